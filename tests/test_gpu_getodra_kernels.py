"""Each Getodra mechanism's kernels alone against the plain function of that mechanism
(tests/plain/getodra_plain.py), at sizes of their own, with inputs made so that a fault shows: inputs of a
convolution before a tile, a portion and a sequence; a value written once and read hundreds of tokens later, or just
before and just after a chunk's edge; one key made to stand out far back, at a page's border and at the query itself;
gates that shut all heads but one."""

import math

import pytest
import torch

from tests.plain import getodra_plain as plain

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


def K():
    from paged_attention_engine_amd.kernels import lib
    return lib


def on_device(flat, width=4):
    return torch.tensor(flat, dtype=torch.int32, device=DEV).view(-1, width)


def step_shape(lens, pasts, bs=16):
    from paged_attention_engine_amd.parts import StepShape

    starts = [sum(lens[:i]) for i in range(len(lens))]
    return StepShape(tuple(range(len(lens))), tuple(starts), tuple(lens), tuple(pasts), bs)


def close(got, want, rel, what):
    got, want = got.double().cpu(), want.double().cpu()
    worst, top = float((got - want).abs().max()), float(want.abs().max())
    assert worst <= rel * top, f"{what}: {worst:.3e} > {rel:.1e} * {top:.3e}"


# ----------------------------------------------------------------------------- the convolution in front of a sublayer


def conv_step(lib, x, dtype, filters, ring, lens, pasts, slots):
    from paged_attention_engine_amd.parts.input_conv import conv_tiles

    lists = conv_tiles(step_shape(lens, pasts), lib.input_conv_tile_rows(filters.shape[1]))
    return lib.input_conv(x.to(DEV), dtype, filters.t().contiguous().to(DEV), ring, on_device(lists["tiles"][0]),
                          on_device(lists["runs"][0]), torch.tensor(slots, dtype=torch.int32, device=DEV))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 6, 8, 9, 12, 30])
@pytest.mark.parametrize("H", [48, 90, 600])
def test_the_convolution_whole_and_in_portions_in_used_slots(dtype, taps, H):
    """Whole, token by token, and in portions around the tile's and the ring's length, in slots in any order that held
    other inputs; two unequal sequences in one step; the rows are the same bits however the sequence was cut."""
    lib = K()
    gen = torch.Generator().manual_seed(taps * 100 + H)
    T = 53
    x = torch.randn((T, H), generator=gen) * 2.0
    filters = torch.randn((H, taps), generator=gen)
    want = plain.with_its_past(x.double(), filters.double())
    rel = 2e-6 if dtype == torch.float32 else 5e-3
    ring = torch.randn((4, max(taps - 1, 1), H), device=DEV) if taps > 1 else None  # what other requests left
    def fresh(slot):
        if ring is not None:
            ring[slot].zero_()  # a slot is zeroed when a request takes it
    fresh(2)
    whole = conv_step(lib, x, dtype, filters, ring, (T,), (0,), [2])
    close(whole, want, rel, f"whole {taps} {H}")
    for cuts in ((1,) * T, (2, 1, 7, 8, 9, 1, 1, 17, 2, 5), (taps, 1, 2, 50), (40, 1, 12)):
        fresh(1)
        at, parts = 0, []
        for n in cuts:
            n = min(n, T - at)
            if n:
                parts.append(conv_step(lib, x[at:at + n], dtype, filters, ring, (n,), (at,), [1]))
            at += n
        assert torch.equal(torch.cat(parts), whole), f"portions {cuts[:4]} {taps} {H}"
    if ring is not None:  # both ways left the same inputs behind
        assert torch.equal(ring[1], ring[2])
        for b in range(1, taps):
            assert torch.equal(ring[1][(T - b) % (taps - 1)].cpu(), x[T - b])
    fresh(3)
    fresh(0)
    both = conv_step(lib, torch.cat([x[:19], x]), dtype, filters, ring, (19, T), (0, 0), [3, 0])
    assert torch.equal(both, torch.cat([whole[:19], whole]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps, H, parts", [(4, 64, 0), (3, 1536, 3), (1, 128, 0), (6, 1028, 2), (2, 4096, 1)])
def test_join_norm_and_convolution_in_one_kernel(dtype, taps, H, parts):
    """Single tokens of five sequences, some in their first positions: the same stream, ring and rows as the norm-and-add
    kernel followed by the convolution, and the plain functions' values."""
    lib = K()
    gen = torch.Generator().manual_seed(H + taps)
    S, eps, scale = 5, 1e-5, 0.7
    pasts = (0, 1, 2, 11, 30)
    history = [torch.randn((n + 1, H), generator=gen) * 2.0 for n in pasts]
    filters = torch.randn((H, taps), generator=gen)
    weight = torch.full((H,), 1.3)
    y = (torch.randn((parts, S, H), generator=gen) if parts else torch.randn((S, H), generator=gen).to(dtype))
    slots = [3, 0, 5, 1, 4]
    ring = torch.zeros((6, max(taps - 1, 1), H), device=DEV) if taps > 1 else None
    for h, slot in zip(history, slots):
        if len(h) > 1:
            conv_step(lib, h[:-1], dtype, filters, ring, (len(h) - 1,), (0,), [slot])
    positions = torch.tensor(pasts, dtype=torch.int32, device=DEV)
    slot_ids = torch.tensor(slots, dtype=torch.int32, device=DEV)
    x = torch.stack([h[-1] for h in history])
    total = y.double().sum(0) if parts else y.double()
    new = x.double() + scale * plain.rms_norm(total, weight.double(), eps)
    want = torch.stack([plain.with_its_past(torch.cat([h[:-1].double(), new[i:i + 1]]), filters.double())[-1]
                        for i, h in enumerate(history)])
    ring2 = None if ring is None else ring.clone()
    res = x.to(DEV)
    rows = lib.norm_join_conv(res, y.to(DEV), weight.to(DEV), eps, scale, dtype, filters.t().contiguous().to(DEV), ring, positions,
                              slot_ids)
    close(res, new, 1e-6, "stream")
    close(rows, want, 2e-6 if dtype == torch.float32 else 5e-3, "rows")
    res2 = x.to(DEV)
    lib.norm_scale_add(res2, y.to(DEV), weight.to(DEV), eps, scale)
    apart = conv_step(lib, res2.cpu(), dtype, filters, ring2, (1,) * S, pasts, slots)
    assert torch.equal(res, res2)
    close(rows, apart, 1e-6 if dtype == torch.float32 else 5e-3, "rows in two kernels")
    if ring is not None:
        assert torch.equal(ring, ring2)


# ----------------------------------------------------------------------------- linear attention with a fixed decay


def decay_plain(proj, gate, norm, decays, H, D, V, eps):
    x = proj.double()
    T = x.shape[0]
    q = plain.silu(x[:, :H * D]).view(T, H, D)
    k = plain.silu(x[:, H * D:2 * H * D]).view(T, H, D)
    v = plain.silu(x[:, 2 * H * D:2 * H * D + H * V]).view(T, H, V)
    o = torch.cat([plain.decaying_readout(q[:, j], k[:, j], v[:, j], decays[j]) for j in range(H)], dim=-1)
    return plain.rms_norm(o, norm.double(), eps) * plain.sigmoid(gate.double())


def decay_step(lib, proj, norm, decays, H, D, V, eps, lens, slots, state):
    """`proj` [rows, 2HD + 2HV] = [q | k | v | gate] of the sequences `lens` one after the other."""
    from paged_attention_engine_amd.parts.delta import runs_and_chunks

    chunk = lib.fixed_decay_chunk(D)
    lists = runs_and_chunks(step_shape(lens, [0] * len(lens)), chunk)
    powers = torch.pow(torch.tensor(decays, dtype=torch.float64)[:, None], torch.arange((chunk or 1) + 1, dtype=torch.float64))
    p = proj.to(DEV)
    out = torch.empty((proj.shape[0], H * V), dtype=proj.dtype, device=DEV)
    lib.fixed_decay_step(p, p[:, 2 * H * D + H * V:2 * H * D + 2 * H * V], out, *(on_device(lists[name][0]) for name in ("serial", "chunks", "scans")),
                         torch.tensor(slots, dtype=torch.int32, device=DEV), powers.float().to(DEV), state, norm.to(DEV), H, D, V, eps)
    return out


SHAPES = [(2, 16, 24), (3, 8, 40), (1, 64, 70), (4, 48, 32), (2, 72, 100), (1, 128, 128), (2, 130, 6), (2, 200, 64), (1, 260, 9),
          (1, 520, 20), (3, 10, 14), (2, 30, 130)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES)
def test_fixed_decays_whole_and_in_steps_in_used_slots(dtype, shape):
    """Every register grouping and both chunk lengths (key widths up to 64, 128, 256, and beyond, which take no chunks),
    widths that are no multiples of four or sixteen; decays of 0, 1, near both and between; a sequence whole, token by token,
    and in portions that cross chunk edges in every way; beside another sequence; in slots that held other state."""
    H, D, V = shape
    lib = K()
    gen = torch.Generator().manual_seed(D * 7 + V)
    T, eps = 149, 1e-5
    decays = [0.9, 1.0, 0.03, 0.0][:H] if D % 3 else [0.999, 0.5, 0.97, 0.1][:H]
    proj = torch.randn((T, 2 * H * D + 2 * H * V), generator=gen).to(dtype)
    norm = (1.0 + 0.2 * torch.randn((H * V,), generator=gen)).to(dtype)
    want = decay_plain(proj, proj[:, 2 * H * D + H * V:], norm, decays, H, D, V, eps)
    rel = 2e-5 if dtype == torch.float32 else 6e-3
    state = torch.randn((4, H, V, D), device=DEV)  # what other requests left
    state[1].zero_()  # a slot is zeroed when a request takes it
    close(decay_step(lib, proj, norm, decays, H, D, V, eps, (T,), [1], state), want, rel, f"whole {shape}")
    whole_state = state[1].clone()
    for cuts in ((1,) * T, (7, 2, 60, 1, 1, 33, 2, 17, 26), (17, 64, 3, 65), (5, 144), (128, 21)):
        state[2].zero_()
        parts, at = [], 0
        for n in cuts:
            parts.append(decay_step(lib, proj[at:at + n], norm, decays, H, D, V, eps, (n,), [2], state))
            at += n
        assert at == T
        close(torch.cat(parts), want, rel, f"steps {cuts[:3]} {shape}")
        close(state[2], whole_state, 2e-5, f"state after steps {shape}")
    # three sequences in one step: a short run, a long one and a single token; the slots are not in order
    for slot in (3, 0, 2):
        state[slot].zero_()
    both = torch.cat([proj[:9], proj[:T], proj[:1]])
    got = decay_step(lib, both, norm, decays, H, D, V, eps, (9, T, 1), [3, 0, 2], state)
    close(got[9:9 + T], want, rel, f"beside others {shape}")
    close(got[:9], want[:9], rel, f"the short run {shape}")
    close(got[9 + T:], want[:1], rel, f"the single token {shape}")
    close(state[0], whole_state, 2e-5, f"state beside others {shape}")


@pytest.mark.parametrize("D, chunk", [(32, 64), (144, 32)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_value_written_once_is_read_across_a_chunks_edge_and_far_back(D, chunk, dtype):
    """One token's key and value alone are not zero; a later token asks for them.  The read-out is the value times the decay
    to the power of the distance, whether the two stand in one chunk, on both sides of an edge, or hundreds of tokens apart."""
    lib = K()
    H, V, T, eps, decay = 1, 16, 6 * chunk + 11, 1e-30, 0.995
    assert lib.fixed_decay_chunk(D) == chunk
    value = torch.linspace(0.5, 2.0, V)
    for wrote, asked in ((chunk - 1, chunk), (chunk, chunk), (chunk, 2 * chunk - 1), (0, chunk - 1), (3, T - 1), (chunk - 1, 5 * chunk),
                         (2 * chunk - 1, 2 * chunk + 1), (T - 2, T - 1), (0, 0)):
        proj = torch.full((T, 2 * H * D + 2 * H * V), -200.0)  # SiLU of -200 is 0
        proj[:, 2 * H * D + H * V:] = 40.0                      # the gate wide open
        proj[wrote, D:2 * D] = 1.0
        proj[wrote, 2 * D:2 * D + V] = value
        proj[asked, :D] = 1.0
        proj = proj.to(dtype)
        state = torch.zeros((1, H, V, D), device=DEV)
        got = decay_step(lib, proj, torch.ones(H * V), [decay], H, D, V, eps, (T,), [0], state)
        one = float(plain.silu(torch.ones(1, dtype=torch.float64)))
        kept = plain.silu(value.to(dtype).double())
        want = plain.rms_norm(kept[None, :], torch.ones((), dtype=torch.float64), 0.0)[0]
        close(got[asked], want, 1e-5 if dtype == torch.float32 else 5e-3, f"{wrote} -> {asked}: direction")
        held = state[0, 0].double().cpu()  # [V, D]: the value times what the decay left of it at the end
        close(held[:, 0], kept * one * decay ** (T - 1 - wrote), 1e-4, f"{wrote}: state at the end")
        others = torch.cat([got[:asked], got[asked + 1:]])
        assert float(others.abs().max()) == 0.0


# ----------------------------------------------------------------------------- latent attention with half rotations and a gate per head


def latent_ways(lib, proj, w, H, D, R, V, C, bs, scale, base, scaling, dtype, new_from, gate):
    """Heads [n, H * V] of the rows from `new_from` on, by the kernel for any shape and, where they take the shape, by the
    matrix-core kernels (single tokens and runs) and with the heads' keys and values formed."""
    from paged_attention_engine_amd.config.model_config import FrequencyRamp, PositionSpec
    from paged_attention_engine_amd.parts.base import POSITION_ENCODINGS
    from paged_attention_engine_amd.parts.latent import expanded_runs, latent_tiles

    T = proj.shape[0]
    ramp = None if scaling is None else FrequencyRamp(**scaling)
    rope = POSITION_ENCODINGS["neox_rope"](PositionSpec(rotary_dim=R, theta=base, ramp=ramp), dtype, DEV)
    positions = torch.arange(T, dtype=torch.int32, device=DEV)
    tok_seq = torch.zeros(T, dtype=torch.int32, device=DEV)
    cos_sin = lib.rope_table(positions, rope.inv_freq)
    pages = -(-T // bs)
    tables = torch.randperm(pages, generator=torch.Generator().manual_seed(T)).to(torch.int32).to(DEV).view(1, -1)
    latent = torch.full((pages + 1, bs, C + R), 3.0, dtype=dtype, device=DEV)  # what other requests left
    cores = lib.latent_attn_supported(dtype, C + R, C, bs)
    latent_t = torch.full((pages + 1, C, bs), 3.0, dtype=dtype, device=DEV) if cores else None
    q_full = torch.empty(T, H * (C + R), dtype=dtype, device=DEV)
    lib.latent_prepare(proj, q_full, H, D, R, R, False, C, w["p.dkv.norm"].to(dtype).to(DEV), 1e-5, cos_sin, positions, tok_seq, tables,
                       latent, latent_t, magnitude=rope.magnitude)
    up_k = w["p.uk"].view(H, D, C).to(dtype).to(DEV)
    up_v = w["p.uv"].view(H, V, C).to(dtype).to(DEV)
    lib.heads_product(q_full.view(T, H, C + R)[:, :, :C], proj[:, :H * (D + R)].view(T, H, D + R)[:, :, :D],
                      up_k.transpose(1, 2).contiguous(), up_k.contiguous())
    n = T - new_from
    ways = {}

    def finish(how, summed):
        heads = torch.empty(n, H * V, dtype=dtype, device=DEV)
        lib.heads_product(heads.view(n, H, V), summed.view(n, H, C), up_v, up_v.transpose(1, 2).contiguous())
        ways[how] = heads

    summed = torch.empty(n, H * C, dtype=dtype, device=DEV)
    lib.paged_attention_masked(summed, q_full[new_from:], latent, None, positions[new_from:], tok_seq[new_from:], tables, H, 1, C + R, C,
                               scale, head_gate=gate[new_from:])
    finish("any shape", summed)
    if cores:
        fast = torch.zeros(n, H * C, dtype=dtype, device=DEV)
        lists = latent_tiles(step_shape((n,), (new_from,), bs), lib.latent_attn_tokens(H, 1), lib.latent_attn_tokens(H, 2))
        for name, column_tiles in (("single", 1), ("runs", 2)):
            if lists[name][0]:
                lib.latent_attn(fast, q_full[new_from:], latent, latent_t, on_device(lists[name][0]), column_tiles, positions[new_from:],
                                tables, H, C, scale, head_gate=gate[new_from:])
        finish("matrix cores", fast)
    if cores and bs % 16 == 0 and lib.latent_key_width(dtype, C + R, C, D + R, V):
        lists = expanded_runs(step_shape((n,), (new_from,), bs), 1)
        heads = torch.zeros(n, H * V, dtype=dtype, device=DEV)
        lib.latent_expanded(heads, proj[new_from:], latent, torch.cat([up_k.view(H * D, C), up_v.view(H * V, C)]),
                            *(on_device(*lists[name]) for name in ("pages", "page_table", "tiles")), positions[new_from:], tables,
                            cos_sin[new_from:].contiguous(), rope.magnitude, H, D, R, R, False, V, C, scale, gate[new_from:])
        ways["keys and values formed"] = heads
    return ways


YARN = dict(factor=8.0, original=64.0, fast=8.0, slow=1.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,R,V,C,bs,T,scaling", [(3, 16, 8, 24, 40, 16, 150, YARN), (2, 24, 16, 8, 16, 8, 70, None),
                                                    (4, 32, 32, 32, 64, 16, 330, YARN), (18, 16, 32, 16, 64, 32, 90, YARN),
                                                    (1, 40, 12, 72, 72, 16, 80, dict(factor=2.0, original=32.0, fast=4.0, slow=0.5)),
                                                    (12, 16, 64, 16, 512, 16, 300, YARN), (5, 40, 32, 64, 96, 16, 210, YARN),
                                                    (2, 128, 64, 128, 512, 16, 170, YARN), (3, 100, 32, 128, 64, 32, 140, None),
                                                    (2, 192, 64, 192, 128, 16, 70, YARN), (1, 96, 32, 64, 160, 48, 100, None)])
@pytest.mark.parametrize("new", ["prompt", "portion", "single"])
def test_latent_attention_with_half_rotations_and_a_gate_per_head(dtype, H, D, R, V, C, bs, T, scaling, new):
    """Projected rows to gated heads against the plain mixer's keys and values formed head by head: pairs (i, i + R / 2), with
    stretched frequencies and the magnitude and without.  One token is made to stand out for the last query: the first of
    the sequence, one on either side of a page's border, one far back in the middle, the query itself."""
    lib = K()
    gen = torch.Generator().manual_seed(T + C)
    randn = lambda *shape, scale=1.0: torch.randn(shape, generator=gen, dtype=torch.float64) * scale
    base, scale = 300.0, 0.2
    mix = {"heads": H, "dim": D, "rot_dim": R, "vdim": V, "kv_rank": C, "scale": scale, "rot": {"base": base, "dims": R}}
    if scaling is not None:
        mix["rot"]["scaling"] = scaling
    w = {"p.q": randn(H * (D + R), 32, scale=0.3), "p.dkv": randn(C + R, 32, scale=0.3), "p.dkv.norm": 1 + randn(C, scale=0.2),
         "p.uk": randn(H * D, C, scale=0.3), "p.uv": randn(H * V, C, scale=0.2), "p.g": randn(H, 32, scale=0.5),
         "p.o": torch.eye(H * V, dtype=torch.float64)}
    w = {name: t.to(dtype).double() for name, t in w.items()}
    new_from = {"prompt": 0, "portion": T - 37, "single": T - 1}[new]
    border = (T - 1) // bs * bs
    for key in sorted({0, border - 1, border, T // 2, T - 1}):
        h = randn(T, 32).to(dtype).double()
        h[key] *= 3.0  # a token whose key part is large
        plain.STORAGE = dtype if dtype == torch.bfloat16 else None
        try:
            want = plain.latent_attention(w, "p.", mix, h, 1e-5, torch.float64, angle_dtype=torch.float32)[new_from:]
        finally:
            plain.STORAGE = None
        wide = (h @ torch.cat([w["p.q"], w["p.dkv"], w["p.g"]]).T).to(dtype).to(DEV)
        gate = wide[:, H * (D + R) + C + R:]
        for how, got in latent_ways(lib, wide, w, H, D, R, V, C, bs, scale, base, scaling, dtype, new_from, gate).items():
            close(got, want, 5e-5 if dtype == torch.float32 else 6e-2, f"{how}, key {key}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,C,R,T", [(4, 64, 32, 300), (18, 64, 32, 40), (3, 40, 8, 90), (2, 128, 32, 150)])
def test_a_gate_that_shuts_every_head_but_one(dtype, H, C, R, T):
    """Gates of -60 leave nothing of a head, a gate of +60 leaves it whole, and 0 halves it: on prompts, on single tokens
    whose keys are split and merged (more than 256 of them), and by the kernel for any shape."""
    lib = K()
    gen = torch.Generator().manual_seed(H)
    D, V, bs = 16, C, 16
    w = {"p.dkv.norm": torch.ones(C, dtype=torch.float64), "p.uk": torch.randn((H * D, C), generator=gen, dtype=torch.float64) * 0.1,
         "p.uv": torch.eye(C, dtype=torch.float64).repeat(H, 1)}
    proj = torch.randn((T, H * (D + R) + C + R), generator=gen).to(dtype).to(DEV)
    for new_from in (0, T - 1):
        gates = {value: torch.full((T, H + 3), value, dtype=dtype, device=DEV)[:, 2:2 + H] for value in (60.0, 0.0)}
        shut = torch.full((T, H + 3), -60.0, dtype=dtype, device=DEV)[:, 2:2 + H]
        shut[:, H - 1] = 60.0
        run = lambda gate: latent_ways(lib, proj, w, H, D, R, V, C, bs, 0.3, 100.0, None, dtype, new_from, gate)
        opened, half, one = run(gates[60.0]), run(gates[0.0]), run(shut)
        for how in opened:
            n = opened[how].shape[0]
            whole = opened[how].view(n, H, V)
            close(half[how].view(n, H, V), 0.5 * whole.double(), 1e-6 if dtype == torch.float32 else 1e-2, f"{how}: half open")
            got = one[how].view(n, H, V)
            assert torch.equal(got[:, H - 1], whole[:, H - 1])
            assert float(got[:, :H - 1].abs().max()) < 1e-20
