"""Getodra on the CPU: the config reader and the plan it gives, the tensors the parts declare, what the layers
keep, the work lists, and the plain implementation pinned by closed forms and by invariants (so that the oracle
the GPU tests compare with is itself checked)."""

import copy
import math

import pytest
import torch

import paged_attention_engine_amd as pae
from paged_attention_engine_amd.config import ConfigError
from tests import getodra_models as M
from tests.plain import getodra_plain as plain


# ----------------------------------------------------------------------------- configuration


def test_the_reader_is_chosen_by_the_architecture_key_and_round_trips():
    for cfg in M.CONFIGS.values():
        typed = pae.read_config_dict(cfg)
        assert type(typed).__name__ == "GetodraConfig"
        assert pae.read_config_dict(typed.to_json_dict()) == typed


def test_every_size_and_constant_comes_from_the_config():
    plan = pae.read_config_dict(M.P).plan()
    assert (plan.hidden_size, plan.vocab_size, plan.head_name, plan.embedding_name) == (64, 300, "head", "embed")
    assert (plan.position_table_name, plan.max_positions, plan.embedding_scale, plan.logit_softcap) == ("pos", 256, 1.0, None)
    # five stops at three layers: two stops use an earlier layer's tensors
    assert [layer.prefix for layer in plan.layers] == ["l0.", "l1.", "l4."]
    assert [e.layer for e in plan.schedule] == [0, 1, 1, 0, 2] and all(e.cache_from is None for e in plan.schedule)
    first, second, third = plan.layers
    for norm, name in ((first.mixer_norm, "norm1"), (first.feed_forward_norm, "norm2"), (plan.final_norm, "final.norm")):
        assert (norm.weight_name, norm.eps, norm.one_weight, norm.size) == (name, 2e-6, True, 64)
    for layer in plan.layers:
        assert layer.arrangement == "branchnorm" and layer.residual_scale == 1.0
        assert (layer.input_conv.taps, layer.input_conv.names) == (4, ("canon1", "canon2"))
    a = second.mixer
    assert (a.kind, a.num_heads, a.nope_dim, a.rope_dim, a.value_dim, a.kv_rank, a.scale, a.window, a.norm_eps, a.gate_name) == (
        "latent_attention", 4, 16, 8, 24, 40, 0.3, None, 2e-6, "g")
    assert (a.position.kind, a.position.rotary_dim, a.position.theta) == ("neox_rope", 8, 500.0)
    assert (a.position.ramp.factor, a.position.ramp.original, a.position.ramp.fast, a.position.ramp.slow) == (8.0, 64.0, 8.0, 1.0)
    g = first.mixer
    assert (g.kind, g.num_heads, g.key_dim, g.value_dim, g.decays, g.norm_eps, g.activation, g.gate_activation) == (
        "fixed_decay_linear_attention", 2, 16, 24, (0.6, 0.995), 2e-6, "silu", "sigmoid")
    d = second.feed_forward
    assert (d.kind, d.intermediate_size, d.activation, d.gate_name, d.weight_suffix) == ("swiglu", 72, "gelu_tanh", "gate", "")
    assert third.feed_forward is None and third.feed_forward_norm is None
    assert set(plan.optional_names) == {"l4.norm2", "l4.canon2"}
    q = pae.read_config_dict(M.Q).plan()
    assert [e.layer for e in q.schedule] == [0, 1, 0, 2, 0]  # a layer that borrows from one that borrows
    assert q.layers[0].mixer.position.ramp is None


def test_declared_tensors_carry_the_designs_names_and_shapes():
    shapes = pae.expected_tensors(pae.read_config_dict(M.P).plan())
    assert shapes["embed"] == (300, 64) and shapes["pos"] == (256, 64) and shapes["head"] == (300, 64)
    for name in ("l0.norm1", "l0.norm2", "l1.norm1", "l4.norm1", "final.norm"):
        assert tuple(shapes[name]) == ()
    assert shapes["l0.canon1"] == (64, 4) and shapes["l0.canon2"] == (64, 4) and shapes["l4.canon1"] == (64, 4)
    assert shapes["l0.mix.q"] == (32, 64) and shapes["l0.mix.k"] == (32, 64) and shapes["l0.mix.v"] == (48, 64)
    assert shapes["l0.mix.g"] == (48, 64) and shapes["l0.mix.o"] == (64, 48) and tuple(shapes["l0.mix.norm"]) == (48,)
    assert shapes["l1.mix.q"] == (96, 64) and shapes["l1.mix.dkv"] == (48, 64) and tuple(shapes["l1.mix.dkv.norm"]) == (40,)
    assert shapes["l1.mix.uk"] == (64, 40) and shapes["l1.mix.uv"] == (96, 40) and shapes["l1.mix.g"] == (4, 64)
    assert shapes["l1.mix.o"] == (64, 96)
    assert shapes["l1.mlp.gate"] == (72, 64) and shapes["l1.mlp.up"] == (72, 64) and shapes["l1.mlp.down"] == (64, 72)
    assert not any(name.startswith(("l2.", "l3.", "l4.mlp.")) or name in ("l4.norm2", "l4.canon2") for name in shapes)


def _damaged(path, value):
    cfg = copy.deepcopy(M.P)
    at = cfg
    for key in path[:-1]:
        at = at[key]
    if value is None:
        at.pop(path[-1])
    else:
        at[path[-1]] = value
    return cfg


@pytest.mark.parametrize("damage, needle", [
    ((("layers", 0, "type"), "windowed"), "unknown layer type"),
    ((("layers", 0, "mixer", "dim"), None), "dim"),
    ((("layers", 0, "mixer", "decay"), None), "decay"),
    ((("layers", 0, "mixer", "decay"), [0.5]), "1 decays for 2 heads"),
    ((("layers", 1, "mixer", "kv_rank"), None), "kv_rank"),
    ((("layers", 1, "mixer", "kv_rank"), 0), "kv_rank"),
    ((("layers", 1, "mixer", "scale"), None), "scale"),
    ((("layers", 1, "mixer", "rot"), None), "rot"),
    ((("layers", 1, "mixer", "rot", "dims"), 7), "rot.dims"),
    ((("layers", 1, "mixer", "rot", "dims"), 10), "rot.dims"),
    ((("layers", 1, "mixer", "rot", "scaling", "slow"), 0.0), "scaling.slow"),
    ((("layers", 1, "mixer", "rot", "scaling", "factor"), None), "factor"),
    ((("layers", 1, "mlp", "kind"), "moe"), "unknown kind"),
    ((("layers", 1, "mlp", "ff"), None), "ff"),
    ((("layers", 2, "weights_of"), 5), "weights_of"),
    ((("layers", 2, "weights_of"), 2), "weights_of"),
    ((("layers", 2, "weights_of"), 0), "differs from layer 0"),
    ((("layers", 1, "weights_of"), 2), "circle"),
    ((("norm",), None), "norm"),
    ((("canon",), None), "canon"),
    ((("canon", "taps"), 0), "canon.taps"),
    ((("max_positions",), None), "max_positions"),
])
def test_a_config_the_engine_cannot_compute_is_refused_with_its_key(damage, needle):
    with pytest.raises(ConfigError, match=needle):
        pae.read_config_dict(_damaged(*damage))


def test_what_the_layers_keep():
    """Every stop has pages or state of its own, also the stops that use another layer's tensors; latent layers keep one
    row a token and no state but the convolutions' inputs; lightning layers one float32 matrix a head and no pages."""
    from paged_attention_engine_amd.engine.model import Model

    model = Model(pae.read_config_dict(M.P).plan(), torch.float32, "meta")
    paged, states = model.cache_specs()
    assert len(paged) == len(states) == 5
    assert paged[0] is None and paged[3] is None and paged[4] is None and paged[1] == paged[2]
    (rows,) = paged[1].tensors
    assert (rows.name, rows.page_shape, paged[1].window) == ("latent", ("page", 48), None)
    kept = [{s.name: (s.shape, s.dtype) for s in stop} for stop in states]
    conv = {"input_conv_0": ((3, 64), torch.float32), "input_conv_1": ((3, 64), torch.float32)}
    assert kept[0] == kept[3] == {"matrices": ((2, 24, 16), torch.float32), **conv}
    assert kept[1] == kept[2] == conv
    assert kept[4] == {"matrices": ((3, 8, 40), torch.float32), "input_conv_0": conv["input_conv_0"]}  # no feed-forward
    cache = model.new_cache(16, 8, 2)
    assert cache.group_of(1) == cache.group_of(2) is not None and cache.group_of(0) is None
    assert cache.state_of(1, "input_conv_1") is not cache.state_of(2, "input_conv_1")
    assert model.graph_safe
    # one tap looks back at nothing
    model = Model(pae.read_config_dict(M.U).plan(), torch.float32, "meta")
    assert model.cache_specs()[1] == [None]


def test_work_lists_of_the_convolutions_and_the_recurrence():
    from paged_attention_engine_amd.parts import StepShape
    from paged_attention_engine_amd.parts.input_conv import conv_tiles
    from paged_attention_engine_amd.parts.delta import SERIAL_ROWS, runs_and_chunks

    shape = StepShape((7, 8, 9), (0, 1, 151), (1, 150, SERIAL_ROWS), (40, 5, 0), 16)
    lists = runs_and_chunks(shape, 64)
    assert lists["serial"] == ([0, 0, 1, 0, 2, 151, SERIAL_ROWS, 0], 4)
    assert lists["chunks"] == ([1, 1, 64, 0, 1, 65, 64, 0, 1, 129, 22, 0], 4)
    assert lists["scans"] == ([1, 0, 3, 22], 4)
    assert runs_and_chunks(StepShape((7,), (0,), (128,), (0,), 16), 64)["scans"] == ([0, 0, 2, 64], 4)  # a whole last chunk
    assert runs_and_chunks(shape, 0) == {"serial": ([0, 0, 1, 0, 1, 1, 150, 0, 2, 151, SERIAL_ROWS, 0], 4), "chunks": ([], 4), "scans": ([], 4)}
    lists = conv_tiles(StepShape((7, 8), (0, 3), (3, 10), (40, 5), 16), 8)
    assert lists["tiles"] == ([0, 0, 3, 0, 1, 3, 8, 0, 1, 11, 2, 8], 4)
    assert lists["runs"] == ([0, 3, 40, 0, 3, 10, 5, 0], 4)


def test_work_lists_of_latent_attention():
    """Single tokens and short runs meet the cached rows as they are; sequences that bring many tokens have all their keys,
    from the sequence's first on, cut into pages of 16 whose rows the heads' keys and values are formed in."""
    from paged_attention_engine_amd.parts import StepShape
    from paged_attention_engine_amd.parts.latent import expanded_runs, latent_tiles

    shape = StepShape((7, 8, 9, 10), (0, 1, 131, 134), (1, 130, 3, 200), (40, 10, 0, 0), 16)
    lists = latent_tiles(shape, 1, 2, 128)
    assert lists["single"] == ([0, 0, 1, 0], 4)
    assert lists["runs"] == ([2, 133, 1, 0, 2, 131, 2, 0], 4)
    formed = expanded_runs(shape, 128)
    pages, _ = formed["pages"]
    assert pages[:8] == [1, 0, 16, 0, 1, 16, 16, 0] and pages[8 * 4:9 * 4] == [1, 128, 12, 0] and pages[9 * 4:10 * 4] == [3, 0, 16, 0]
    assert len(pages) // 4 == 9 + 13
    table, width = formed["page_table"]
    assert width == 13 and table == list(range(9)) + [-1] * 4 + list(range(9, 22))
    # pieces of 64 tokens, those with the most keys first, by their row in the table of pages
    assert formed["tiles"] == ([1, 326, 8, 1, 262, 64, 0, 129, 2, 0, 65, 64, 1, 198, 64, 0, 1, 64, 1, 134, 64], 3)
    assert latent_tiles(shape, 1, 2)["runs"][0][:4] == [3, 332, 2, 0]  # without the other kind every run is here
    assert expanded_runs(StepShape((7,), (0,), (5,), (9,), 16), 128) == {"pages": ([], 4), "page_table": ([], 1), "tiles": ([], 3)}


def test_the_bench_shape_is_a_config_the_reader_takes():
    """`bench.py --design getodra` builds its model from a config of its own making: as many layers as asked for."""
    import bench

    for layers in (1, 2, 8):
        plan = pae.read_config_dict(bench.getodra_shape(bench.QWEN25_1P5B, layers)).plan()
        assert len(plan.schedule) == layers and plan.hidden_size == 1536
    assert [e.layer for e in plan.schedule] == [0, 1, 2, 3, 4, 3, 5, 6]
    assert {layer.mixer.kind for layer in plan.layers} == {"latent_attention", "fixed_decay_linear_attention"}
    assert all(0.5 < d < 1.0 for d in plan.layers[0].mixer.decays)


# ----------------------------------------------------------------------------- the plain implementation, pinned


def test_norm_and_activations_by_closed_forms():
    x = torch.tensor([[3.0, -4.0]], dtype=torch.float64)
    root = math.sqrt(12.5 + 0.5)
    got = plain.rms_norm(x, torch.tensor(2.0, dtype=torch.float64), 0.5)  # one number for both features
    assert torch.allclose(got, torch.tensor([[6.0 / root, -8.0 / root]], dtype=torch.float64))
    z = torch.tensor([0.0, 1.0, -2.0], dtype=torch.float64)
    assert torch.allclose(plain.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert torch.allclose(plain.silu(z), torch.nn.functional.silu(z))


def test_a_convolution_by_hand():
    """Two channels, three taps: the last tap weighs the token itself, the first the token two back."""
    x = torch.tensor([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0], [4.0, 40.0]], dtype=torch.float64)
    f = torch.tensor([[0.5, 0.25, 2.0], [0.0, 1.0, 0.0]], dtype=torch.float64)
    got = plain.with_its_past(x, f)
    want = [[1 + 2 * 1, 10 + 0], [2 + 2 * 2 + 0.25 * 1, 20 + 10], [3 + 2 * 3 + 0.25 * 2 + 0.5 * 1, 30 + 20],
            [4 + 2 * 4 + 0.25 * 3 + 0.5 * 2, 40 + 30]]
    assert torch.allclose(got, torch.tensor(want, dtype=torch.float64))
    assert torch.allclose(plain.with_its_past(x, f[:, 2:]), x * (1.0 + f[:, 2]))  # one tap


def test_stretched_frequencies_by_hand():
    """dims 8, base 500, original 64: a pair makes 8 turns at index 8 ln(64 / (16 pi)) / (2 ln 500) = 0.155 (rounded down: 0)
    and 1 turn at 8 ln(64 / (2 pi)) / (2 ln 500) = 1.494 (rounded up: 2); the first pair keeps its frequency, the second is
    blended half and half, the others are divided by the factor."""
    rot = {"dims": 8, "base": 500.0, "scaling": {"factor": 8.0, "original": 64, "fast": 8.0, "slow": 1.0}}
    f = [500.0 ** (-i / 4.0) for i in range(4)]
    want = [f[0], 0.5 * f[1] / 8.0 + 0.5 * f[1], f[2] / 8.0, f[3] / 8.0]
    got, magnitude = plain.stretched_frequencies(rot)
    assert torch.allclose(got, torch.tensor(want, dtype=torch.float64), rtol=1e-12)
    assert math.isclose(magnitude, 0.1 * math.log(8.0) + 1.0)
    plainly, one = plain.stretched_frequencies({"dims": 8, "base": 500.0})
    assert torch.allclose(plainly, torch.tensor(f, dtype=torch.float64), rtol=1e-12) and one == 1.0
    # the product's own rotation has these frequencies and this magnitude
    from paged_attention_engine_amd.config.model_config import FrequencyRamp, PositionSpec
    from paged_attention_engine_amd.parts.base import POSITION_ENCODINGS
    mine = POSITION_ENCODINGS["neox_rope"](PositionSpec(rotary_dim=8, theta=500.0, ramp=FrequencyRamp(8.0, 64.0, 8.0, 1.0)),
                                           torch.float32, "cpu")
    assert math.isclose(mine.magnitude, magnitude) and torch.allclose(mine.inv_freq.double(), got, rtol=1e-6)


def test_a_rotated_pair_by_hand():
    """Features (i, i + n) turn together, both times the magnitude; the features behind pass as they are."""
    x = torch.zeros((3, 1, 6), dtype=torch.float64)
    x[:, 0, 1], x[:, 0, 3], x[:, 0, 4] = 1.0, 2.0, 7.0
    got = plain.rotate_halves(x, torch.tensor([0.3, 0.5], dtype=torch.float64), 1.5)
    for t in range(3):
        c, s = 1.5 * math.cos(0.5 * t), 1.5 * math.sin(0.5 * t)
        assert torch.allclose(got[t, 0, [1, 3]], torch.tensor([c - 2 * s, 2 * c + s], dtype=torch.float64))
    keep = plain.rotate_halves(x, torch.tensor([0.3], dtype=torch.float64), 1.5)
    assert torch.equal(keep[..., 2:], x[..., 2:])


def test_causal_softmax_on_flat_scores_and_with_one_key():
    T = 6
    v = torch.arange(T, dtype=torch.float64)[:, None]
    got = plain.causal_softmax(torch.zeros((T, 3), dtype=torch.float64), torch.randn((T, 3), dtype=torch.float64), v, 0.5)
    assert torch.allclose(got[:, 0], torch.arange(T, dtype=torch.float64) / 2.0)  # the mean of 0 .. i
    assert float(got[0, 0]) == 0.0


def test_two_steps_of_the_decaying_state_by_hand():
    q = torch.tensor([[1.0, 0.0], [1.0, 1.0]], dtype=torch.float64)
    k = torch.tensor([[2.0, 1.0], [0.0, 3.0]], dtype=torch.float64)
    v = torch.tensor([[5.0], [7.0]], dtype=torch.float64)
    # S1 = k1 v1 = [10, 5]; o1 = 10.  S2 = 0.5 S1 + [0, 21] = [5, 23.5]; o2 = 28.5
    assert torch.allclose(plain.decaying_readout(q, k, v, 0.5), torch.tensor([[10.0], [28.5]], dtype=torch.float64))


def test_the_layer_whose_tensors_a_layer_uses():
    assert [plain.owner_of(M.Q, i) for i in range(5)] == [0, 1, 0, 3, 0]
    assert [plain.owner_of(M.P, i) for i in range(5)] == [0, 1, 1, 0, 4]


# ----------------------------------------------------------------------------- a mechanism left out shows


@pytest.fixture(scope="module")
def model_p(tmp_path_factory):
    cfg, weights = M.read_folder(M.make_folder(tmp_path_factory.mktemp("getodra_cpu"), "P"))
    tokens = M.tokens_for("P", 40)
    return cfg, weights, tokens, plain.forward(weights, cfg, tokens, torch.float64)


def _moved(model_p, change) -> float:
    """How far the logits move, in units of the float32 tests' bound, under a changed config or changed weights."""
    cfg, weights, tokens, want = model_p
    cfg2, weights2 = copy.deepcopy(cfg), dict(weights)
    change(cfg2, weights2)
    got = plain.forward(weights2, cfg2, tokens, torch.float64)
    return float((got - want).abs().max()) / (1e-4 * float(want.abs().max()))


def _zeroed(name):
    return lambda c, w: w.update({name: torch.zeros_like(w[name])})


@pytest.mark.parametrize("what, change", [
    ("no positions", _zeroed("pos")),
    ("no convolution in front of a mixer", _zeroed("l0.canon1")),
    ("no convolution in front of a feed-forward", _zeroed("l1.canon2")),
    ("the filters the other way round", lambda c, w: w.update({"l0.canon1": w["l0.canon1"].flip(1)})),
    ("the norm after the mixer left at one", lambda c, w: w.update({"l1.norm1": torch.ones_like(w["l1.norm1"])})),
    ("the latent's norm left at one", lambda c, w: w.update({"l1.mix.dkv.norm": torch.ones_like(w["l1.mix.dkv.norm"])})),
    ("the lightning norm left at one", lambda c, w: w.update({"l0.mix.norm": torch.ones_like(w["l0.mix.norm"])})),
    ("no gate on the latent's heads (all half open)", _zeroed("l1.mix.g")),
    ("no gate on the lightning heads", _zeroed("l0.mix.g")),
    ("frequencies not stretched", lambda c, w: [c["layers"][i]["mixer"]["rot"].pop("scaling") for i in (1, 2)]),
    ("another original context", lambda c, w: [c["layers"][i]["mixer"]["rot"]["scaling"].update(original=256) for i in (1, 2)]),
    ("another scale", lambda c, w: [c["layers"][i]["mixer"].update(scale=0.31) for i in (1, 2)]),
    ("a decay off in the third place", lambda c, w: c["layers"][0]["mixer"].update(decay=[0.6, 0.99])),
    ("the decays swapped", lambda c, w: c["layers"][0]["mixer"].update(decay=[0.995, 0.6])),
    ("the borrowing layer with other tensors", lambda c, w: c["layers"][3].update(weights_of=None) or [
        w.update({"l3." + n[3:]: t * 1.05}) for n, t in list(w.items()) if n.startswith("l0.")]),
])
def test_a_mechanism_left_out_or_a_constant_off_moves_the_logits(model_p, what, change):
    assert _moved(model_p, change) > 10.0, what


def test_a_far_token_shows(model_p):
    """The first token of forty, changed, moves the last token's logits: the state and the latent rows reach back."""
    cfg, weights, tokens, want = model_p
    other = [(tokens[0] + 1) % cfg["vocab"]] + tokens[1:]
    got = plain.forward(weights, cfg, other, torch.float64)
    assert float((got[-1] - want[-1]).abs().max()) > 10.0 * 1e-4 * float(want.abs().max())
