"""A short convolution over time in front of a sublayer: what the sublayer reads is the stream plus a causal
convolution of it, channel by channel,

    h_t + sum_j w[:, j] h_(t - taps + 1 + j),   zeros before the sequence's first token.

The last taps - 1 inputs of a request are state, kept in float32 as a ring (the input at position p in row
p % (taps - 1)), so that a prompt may be cut anywhere and a decoded token writes one row.  The block that owns the
convolution hands it the float32 stream; sums are float32 and the result is rounded once.  In steps of single tokens the
convolution can ride in the kernel that joins the sublayer before (`kernels.lib.norm_join_conv`)."""

from __future__ import annotations

import torch

from ..cache.manager import StateSpec
from ..kernels import lib as K
from .base import Part, StepShape
from .delta import sequence_runs


def conv_tiles(shape: StepShape, rows: int):
    """Pieces of up to `rows` rows: (table row of the sequence, first flat row, rows, rows of the sequence before)."""
    tiles = []
    for row, (start, n) in enumerate(zip(shape.q_starts, shape.q_lens)):
        for at in range(0, n, rows):
            tiles += [row, start + at, min(rows, n - at), at]
    return {"tiles": (tiles, 4), **sequence_runs(shape)}


class InputConv(Part):
    graph_safe = True

    def __init__(self, spec, which: int, hidden_size: int, dtype, device):
        """`which`: 0 in front of the mixer, 1 in front of the feed-forward."""
        super().__init__(spec, dtype, device)
        if not 1 <= spec.taps <= 64:
            raise ValueError(f"a convolution of {spec.taps} taps (the kernels take 1..64)")
        self.name = spec.names[which]
        self.state_name = f"input_conv_{which}"
        self.hidden_size = hidden_size

    def tensors(self, prefix):
        return {prefix + self.name: (self.hidden_size, self.spec.taps)}

    def bind(self, prefix, weights):
        # float32 like the sums, tap by tap
        self.filters = weights[prefix + self.name].to(device=self.device, dtype=torch.float32).t().contiguous()

    def state_spec(self):
        if self.spec.taps == 1:
            return None  # a convolution of one tap looks back at nothing
        return StateSpec((self.spec.taps - 1, self.hidden_size), torch.float32, self.state_name)

    def step_lists_key(self, block_size: int):
        return ("tiles of an input convolution", K.input_conv_tile_rows(self.spec.taps))

    def step_lists(self, shape: StepShape):
        return conv_tiles(shape, K.input_conv_tile_rows(self.spec.taps))

    def ring(self, ctx, entry: int):
        """The requests' last inputs at stop `entry` (None: nothing is kept)."""
        return None if self.spec.taps == 1 else ctx.cache.state_of(entry, self.state_name)

    def forward(self, ctx, residual: torch.Tensor, entry: int) -> torch.Tensor:
        lists = ctx.memo[self.step_lists_key(ctx.cache.block_size)]
        return K.input_conv(residual, self.dtype, self.filters, self.ring(ctx, entry), lists["tiles"], lists["runs"], ctx.slots)

    def join_and_forward(self, ctx, residual: torch.Tensor, y: torch.Tensor, norm, scale: float, entry: int) -> torch.Tensor:
        """For a step of single tokens: residual += scale * norm(y), then `forward`, in one kernel."""
        return K.norm_join_conv(residual, y, norm.weight, norm.spec.eps, scale, self.dtype, self.filters, self.ring(ctx, entry),
                                ctx.positions, ctx.slots)
