"""Mulenex on the CPU: the config reader and the plan it gives, the tensors the parts declare, what the layers keep in
the cache, and the plain implementation pinned by closed forms and by invariants (so that the oracle the GPU tests
compare with is itself checked)."""

import copy
import math

import pytest
import torch

import paged_attention_engine_amd as pae
from paged_attention_engine_amd.config import ConfigError
from tests import mulenex_models as M
from tests.plain import mulenex_plain as plain

F64 = torch.float64


# ----------------------------------------------------------------------------- configuration


def test_the_reader_is_chosen_by_the_architecture_key_and_round_trips():
    assert "Mulenex" in pae.known_architectures()
    for cfg in M.CONFIGS.values():
        typed = pae.read_config_dict(cfg)
        assert type(typed).__name__ == "MulenexConfig"
        assert pae.read_config_dict(typed.to_json_dict()) == typed


def test_every_size_and_constant_comes_from_the_config():
    plan = pae.read_config_dict(M.P).plan()
    assert (plan.hidden_size, plan.vocab_size, plan.head_name, plan.embedding_name) == (64, 300, "head", "embed")
    assert plan.sinusoid_base == 10000.0 and plan.embedding_scale == 1.0 and plan.max_positions is None
    assert [(e.layer, e.cache_from) for e in plan.schedule] == [(i, None) for i in range(4)]
    first, second, third, fourth = plan.layers
    for layer in plan.layers:
        assert layer.arrangement == "sandwich"
        norms = [layer.mixer_norm, layer.mixer_out_norm] + ([] if layer.feed_forward is None else [layer.feed_forward_norm, layer.feed_forward_out_norm])
        assert all(n.weight_offset == 1.0 and n.eps == 2e-6 for n in norms)
    a = first.mixer
    assert (a.kind, a.num_heads, a.num_kv_heads, a.head_dim, a.v_dim, a.scale, a.softcap, a.qk_norm, a.qk_norm_eps, a.head_gate_name) == (
        "attention", 4, 2, 16, 24, 0.3, 5.0, "per_head", 2e-6, "g")
    assert (a.temperature.coef, a.temperature.every, a.value_mix, a.window, a.position) == (0.5, 7, "source", None, None)
    assert not (a.qkv_bias or a.out_bias or a.sinks or a.plain or a.convolved)
    e = first.feed_forward
    assert (e.kind, e.intermediate_size, e.num_experts, e.top, e.groups, e.route_scale, e.activation, e.weights_over, e.router_bias_name) == (
        "experts", 24, 6, 2, 1, 1.0, "silu", "chosen", "router.b")
    assert (e.shared.intermediate_size, e.shared.prefix, e.shared.gate_name) == (40, "shared.", "sg")
    m = second.mixer
    assert (m.kind, m.num_heads, m.key_dim, m.value_dim, m.gate_cap, m.norm_eps, m.readout_floor) == ("matrix_memory", 2, 16, 24, 8.0, 2e-6, 1e-6)
    d = second.feed_forward
    assert (d.kind, d.intermediate_size, d.activation, d.bias, d.bias_suffix) == ("dense", 88, "relu2", True, ".b")
    assert third.mixer.value_mix == "mixed" and third.mixer.softcap is None and third.mixer.temperature is None
    assert third.feed_forward.shared is None
    assert fourth.mixer.value_mix is None and fourth.feed_forward is None
    # only the first layer with v_mix is the source, wherever it stands
    q = pae.read_config_dict(M.Q).plan()
    assert [getattr(layer.mixer, "value_mix", None) for layer in q.layers] == [None, None, "source", None, "mixed", "mixed"]


def test_declared_tensors_carry_the_designs_names_and_shapes():
    plan = pae.read_config_dict(M.P).plan()
    shapes = pae.expected_tensors(plan)
    assert shapes["embed"] == (300, 64) and shapes["head"] == (300, 64) and tuple(shapes["final.norm"]) == (64,)
    assert all(tuple(shapes[f"l0.{name}"]) == (64,) for name in ("norm1", "norm1b", "norm2", "norm2b"))
    assert shapes["l0.mix.q"] == (64, 64) and shapes["l0.mix.k"] == (32, 64) and shapes["l0.mix.v"] == (48, 64)
    assert tuple(shapes["l0.mix.q.norm"]) == (16,) and tuple(shapes["l0.mix.k.norm"]) == (16,)
    assert shapes["l0.mix.g"] == (4, 64) and shapes["l0.mix.o"] == (64, 96)
    assert "l0.mix.vmix" not in shapes and "l0.mix.vmix" in plan.optional_names  # stored or not, the source mixes nothing
    assert shapes["l2.mix.vmix"] == () and "l3.mix.vmix" in plan.optional_names
    assert shapes["l1.mix.q"] == (32, 64) and shapes["l1.mix.v"] == (48, 64) and shapes["l1.mix.g"] == (48, 64)
    assert shapes["l1.mix.i"] == (2, 64) and shapes["l1.mix.f.b"] == (2,) and tuple(shapes["l1.mix.norm"]) == (48,)
    assert shapes["l1.mlp.up"] == (88, 64) and shapes["l1.mlp.up.b"] == (88,) and shapes["l1.mlp.down.b"] == (64,)
    assert shapes["l0.mlp.router"] == (6, 64) and shapes["l0.mlp.router.b"] == (6,) and shapes["l0.mlp.e5.gate"] == (24, 64)
    assert shapes["l0.mlp.shared.up"] == (40, 64) and shapes["l0.mlp.shared.down"] == (64, 40) and shapes["l0.mlp.shared.sg"] == (1, 64)
    assert "l2.mlp.shared.up" not in shapes and "l3.norm2" not in shapes and "l3.norm2" in plan.optional_names


def _damaged(path, value, cfg=None):
    cfg = copy.deepcopy(cfg or M.P)
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
    ((("layers", 0, "mixer", "kv_heads"), 3), "not a multiple"),
    ((("layers", 0, "mixer", "scale"), None), "scale"),
    ((("layers", 0, "mixer", "vdim"), "wide"), "vdim"),
    ((("layers", 0, "mixer", "softcap"), -1.0), "softcap"),
    ((("layers", 0, "mixer", "q_temp", "every"), 0), "every"),
    ((("layers", 0, "mixer", "q_temp", "coef"), None), "coef"),
    ((("layers", 2, "mixer", "vdim"), 16), "cannot be mixed"),
    ((("layers", 2, "mixer", "kv_heads"), 3), "cannot be mixed"),
    ((("layers", 1, "mixer", "gate_cap"), 0.0), "gate_cap"),
    ((("layers", 1, "mixer", "dim"), None), "dim"),
    ((("layers", 1, "mlp", "ff"), 0), "ff"),
    ((("layers", 0, "mlp", "kind"), "wide"), "unknown kind"),
    ((("layers", 0, "mlp", "router", "top"), 7), "top"),
    ((("layers", 0, "mlp", "expert"), None), "expert"),
    ((("layers", 0, "mlp", "shared"), {"wide": 3}), "ff"),
    ((("norm",), None), "norm"),
    ((("vocab",), None), "vocab"),
])
def test_a_faulty_config_is_refused_with_the_key_named(damage, needle):
    with pytest.raises(ConfigError, match=needle):
        pae.read_config_dict(_damaged(*damage))


def test_random_weights_make_a_folder_the_loader_accepts(tmp_path):
    folder = M.make_folder(tmp_path, "P")
    cfg, tensors = M.read_folder(folder)
    plan = pae.read_config(folder).plan()
    declared = pae.expected_tensors(plan)
    assert cfg["architecture"] == "Mulenex" and set(tensors) == set(declared)
    got = pae.load_weights(folder, declared, plan.optional_names)
    assert torch.equal(got["l0.mlp.shared.down"], tensors["l0.mlp.shared.down"]) and got["l2.mix.vmix"].shape == ()
    assert float(tensors["l0.norm1b"].float().abs().mean()) < 0.5   # stored around zero
    assert float(tensors["l0.mix.q.norm"].float().mean()) > 0.5     # a plain weight


def test_what_the_layers_keep():
    """An attention keeps keys and values for ever, a memory its matrix (with the key sum as one more row) and its maximum."""
    model = pae.Model(pae.read_config_dict(M.P).plan(), torch.float32, "cpu")
    paged, states = model.cache_specs()
    assert [t.name for t in paged[0].tensors] == ["k", "v"] and paged[0].window is None
    assert paged[0].tensors[0].shape(16) == (2, 16, 16) and paged[0].tensors[1].shape(16) == (2, 24, 16)
    assert states[0] is None and paged[1] is None
    assert {s.name: s.shape for s in states[1]} == {"memory": (2, 25, 16), "memory_max": (2,)}
    cache = model.new_cache(16, 8, 2)
    assert cache.group_of(1) is None and cache.group_of(0) != cache.group_of(3)
    assert cache.create_sequence(1) and cache.reserve(1, 100).ok and cache.release_passed(1) == 0
    assert model.graph_safe
    paged, states = pae.Model(pae.read_config_dict(M.V).plan(), torch.float32, "cpu").cache_specs()
    assert paged == [None, None] and states[0][0].shape == (1, 41, 136)


def test_specs_that_do_not_go_together_are_refused():
    from paged_attention_engine_amd.config.model_config import ExpertsSpec, MixerSpec, QueryTemperature, SharedExpertSpec
    from paged_attention_engine_amd.parts import MIXERS, FEED_FORWARDS, build_part

    mixer = lambda **kw: build_part(MIXERS, "mixer", MixerSpec(hidden_size=8, num_heads=2, num_kv_heads=1, head_dim=4, **kw), torch.float32, "cpu")
    experts = lambda **kw: build_part(FEED_FORWARDS, "feed-forward", ExpertsSpec(hidden_size=8, intermediate_size=4, num_experts=4, **kw),
                                      torch.float32, "cpu")
    with pytest.raises(ValueError, match="value_mix"):
        mixer(value_mix="third")
    with pytest.raises(ValueError, match="temperature"):
        mixer(temperature=QueryTemperature(0.1, 0))
    with pytest.raises(ValueError, match="gate per head"):
        mixer(qk_norm="head", head_gate_name="g")
    with pytest.raises(ValueError, match="one group"):
        experts(weights_over="chosen", groups=2)
    with pytest.raises(ValueError, match="weights_over"):
        experts(weights_over="some")
    with pytest.raises(ValueError, match="shared"):
        experts(shared=SharedExpertSpec(0))
    assert experts(shared=SharedExpertSpec(9)).shared_pieces == 3


# ----------------------------------------------------------------------------- the plain implementation


def test_position_vectors_by_hand():
    got = plain.position_vectors(4, 6)
    assert torch.equal(got[0], torch.tensor([0.0, 1.0, 0.0, 1.0, 0.0, 1.0], dtype=F64))
    a = [3.0, 3.0 * 10000.0 ** (-2 / 6), 3.0 * 10000.0 ** (-4 / 6)]
    want = [f(x) for x in a for f in (math.sin, math.cos)]
    assert torch.allclose(got[3], torch.tensor(want, dtype=F64))


def test_norm_and_activation_by_hand():
    x = torch.tensor([[3.0, 4.0]], dtype=F64)
    root = math.sqrt(12.5 + 0.5)
    got = plain.offset_norm(x, torch.tensor([0.5, -1.0], dtype=F64), 0.5)
    assert torch.allclose(got, torch.tensor([[3.0 / root * 1.5, 0.0]], dtype=F64))
    assert plain.relu_squared(torch.tensor([-2.0, 0.0, 3.0])).tolist() == [0.0, 0.0, 9.0]
    z = torch.tensor([-50.0, -1.0, 0.0, 2.0, 50.0], dtype=F64)
    assert torch.allclose(plain.log_sigmoid(z), torch.log(plain.sigmoid(z)))


def test_the_query_temperature_steps_where_it_should():
    got = plain.query_temperature(10, {"coef": 0.5, "every": 4})
    ln = math.log
    # floor((p + 1) / 4): 0 for p = 0..2, 1 for p = 3..6, 2 for p = 7..9
    want = [1.0] * 3 + [1 + 0.5 * ln(2)] * 4 + [1 + 0.5 * ln(3)] * 3
    assert torch.allclose(got, torch.tensor(want, dtype=F64))
    assert torch.equal(plain.query_temperature(3, None), torch.ones(3, dtype=F64))


def test_attention_is_causal_and_its_cap_bends_the_scores():
    """Two keys, scores 0 and s: the weights are those of the capped score; grouped heads read their own keys."""
    q = torch.tensor([[[1.0], [1.0]], [[2.0], [1.0]]], dtype=F64)   # [T = 2, H = 2, D = 1]
    k = torch.tensor([[[0.0], [0.0]], [[3.0], [0.0]]], dtype=F64)   # [T, G = 2, D]
    v = torch.tensor([[[1.0], [10.0]], [[5.0], [20.0]]], dtype=F64)
    got = plain.capped_softmax_attend(q, k, v, 0.5, 2.0)
    assert float(got[0, 0, 0]) == 1.0 and float(got[0, 1, 0]) == 10.0    # a token's first sees itself alone
    s = 2.0 * math.tanh(2.0 * 3.0 * 0.5 / 2.0)
    w = math.exp(s) / (1.0 + math.exp(s))
    assert math.isclose(float(got[1, 0, 0]), (1 - w) * 1.0 + w * 5.0, rel_tol=1e-12)
    assert math.isclose(float(got[1, 1, 0]), 15.0, rel_tol=1e-12)         # flat scores
    free = plain.capped_softmax_attend(q, k, v, 0.5, None)
    w = math.exp(3.0) / (1.0 + math.exp(3.0))
    assert math.isclose(float(free[1, 0, 0]), (1 - w) * 1.0 + w * 5.0, rel_tol=1e-12)


def test_value_mixing_by_hand():
    own, first = torch.tensor([2.0], dtype=F64), torch.tensor([10.0], dtype=F64)
    assert float(plain.mix_values(own, first, torch.tensor(0.25, dtype=F64))) == 0.75 * 2 + 0.25 * 10
    assert plain.first_mixing_layer(M.Q) == 2 and plain.first_mixing_layer(M.V) is None


def test_two_steps_of_the_matrix_memory_by_hand():
    q = torch.tensor([[[1.0, 0.0]], [[0.0, 2.0]]], dtype=F64)
    k = torch.tensor([[[1.0, 1.0]], [[0.0, 1.0]]], dtype=F64)
    v = torch.tensor([[[2.0]], [[-4.0]]], dtype=F64)
    log_in = torch.tensor([[-1.0], [0.5]], dtype=F64)
    log_keep = torch.tensor([[-0.2], [-0.3]], dtype=F64)
    got = plain.matrix_memory_recurrence(q, k, v, log_in, log_keep)
    # step 1: m = max(-0.2 + 0, -1) = -0.2 (the maximum starts at 0: from minus infinity it would be -1)
    take1 = math.exp(-0.8)
    assert math.isclose(float(got[0, 0, 0]), take1 * 2.0 / (max(take1, math.exp(0.2)) + 1e-6), rel_tol=1e-12)
    # step 2: m = max(-0.3 - 0.2, 0.5) = 0.5; keep = e^-1.0; take = 1
    keep2 = math.exp(-1.0)
    row2, n2 = keep2 * take1 * 2.0 + 1.0 * -4.0, keep2 * take1 + 1.0
    assert math.isclose(float(got[1, 0, 0]), 2 * row2 / (max(abs(2 * n2), math.exp(-0.5)) + 1e-6), rel_tol=1e-12)


def test_routing_weighs_the_chosen_logits_alone():
    z = torch.tensor([[1.0, 3.0, 2.0, -5.0]], dtype=F64)
    margins = []
    chosen, weights = plain.route(z, 2, margins)
    assert chosen.tolist() == [[1, 2]] and math.isclose(float(margins[0][0]), 1.0)
    w = 1.0 / (1.0 + math.exp(-1.0))
    assert torch.allclose(weights, torch.tensor([[w, 1.0 - w]], dtype=F64))
    _, weights = plain.route(z, 1)
    assert weights.tolist() == [[1.0]]


def test_the_test_models_show_mistakes(tmp_path):
    """Leaving a mechanism out, or getting a constant one off, moves a test model's logits far beyond the tests' bounds."""
    folder = M.make_folder(tmp_path, "P")
    cfg, weights = M.read_folder(folder)
    tokens = M.tokens_for("P", 40)
    right = plain.forward(weights, cfg, tokens, F64)
    top = float(right.abs().max())

    def moved(cfg2=None, weights2=None, **patch):
        saved = {name: getattr(plain, name) for name in patch}
        for name, fn in patch.items():
            setattr(plain, name, fn)
        try:
            other = plain.forward(weights2 or weights, cfg2 or cfg, tokens, F64)
        finally:
            for name, fn in saved.items():
                setattr(plain, name, fn)
        return float((other - right).abs().max()) / top

    def with_key(path, value):
        return _damaged(path, value, cfg)

    bound = 1e-3
    assert moved(with_key(("layers", 0, "mixer", "softcap"), None)) > bound
    assert moved(with_key(("layers", 0, "mixer", "softcap"), 5.5)) > bound
    assert moved(with_key(("layers", 0, "mixer", "q_temp", "every"), 8)) > bound            # the temperature steps later
    assert moved(with_key(("layers", 0, "mixer", "q_temp"), None)) > bound
    assert moved(with_key(("layers", 2, "mixer", "v_mix"), False)) > bound                  # values not mixed
    assert moved(with_key(("layers", 1, "mixer", "gate_cap"), 7.0)) > bound
    assert moved(with_key(("layers", 0, "mlp", "router", "top"), 3)) > bound
    assert moved(with_key(("layers", 0, "mlp", "shared"), None)) > bound
    assert moved(mix_values=lambda own, first, share: share * own + (1.0 - share) * first) > bound   # the share on the other side
    assert moved(chosen_softmax=lambda z, chosen: torch.softmax(z, -1).gather(1, chosen)) > bound   # the softmax over all
    assert moved(offset_norm=lambda x, w, eps: plain.over_rms(x, eps) * w) > bound                  # the weight without its one
    assert moved(relu_squared=lambda z: torch.clamp(z, min=0.0)) > bound
    assert moved(position_vectors=lambda n, width: torch.zeros((n, width), dtype=F64)) > bound
    vectors = plain.position_vectors(40, 64)
    halves = torch.cat([vectors[:, 0::2], vectors[:, 1::2]], dim=1)
    assert moved(position_vectors=lambda n, width: halves) > bound                                  # all sines before all cosines
    assert moved(READOUT_FLOOR=1.0) > 2e-4   # (against rounding's 1e-5)
    ones = lambda *names: {**weights, **{n: torch.ones_like(weights[n]) for n in names}}
    zeros = lambda *names: {**weights, **{n: torch.zeros_like(weights[n]) for n in names}}
    assert moved(weights2=ones("l0.mix.q.norm")) > bound and moved(weights2=ones("l3.mix.k.norm")) > bound
    assert moved(weights2=zeros("l0.mix.g")) > bound        # every head's gate at a half
    assert moved(weights2=zeros("l0.mlp.router.b")) > bound and moved(weights2=zeros("l0.mlp.shared.sg")) > bound
    assert moved(weights2=zeros("l1.mlp.up.b")) > bound and moved(weights2=zeros("l1.mlp.down.b")) > bound
    assert moved(weights2=zeros("l0.norm1b")) > bound and moved(weights2=zeros("l2.norm2b")) > bound
    assert moved(weights2=zeros("l1.mix.i.b")) > bound and moved(weights2=zeros("l1.mix.f.b")) > bound
