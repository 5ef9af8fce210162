"""Each Mulenex mechanism's kernels alone against the plain function of that mechanism
(tests/plain/mulenex_plain.py), at sizes of their own, with inputs made so that a fault shows: positions far out; a
temperature at the positions where it steps; one key made to stand out far back, at a page's border and at the query
itself, with scores on the bend of the cap; gates that shut all heads but one; a value written into the memory once
and read hundreds of tokens later, or just before and just after a chunk's edge; logits too large to exponentiate."""

import math

import pytest
import torch

from tests.plain import mulenex_plain as plain

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


# ----------------------------------------------------------------------------- embedding with sinusoids


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [6, 64, 75, 600])
def test_sinusoids_of_any_position_join_the_embedding(dtype, width):
    """Positions in any order and far out (an angle of float32 precision would be off by thousandths at 100,000)."""
    gen = torch.Generator().manual_seed(width)
    vocab = 40
    table = torch.randn((vocab, width), generator=gen).to(dtype)
    positions = torch.tensor([0, 1, 2, 511, 100003, 7, 65536], dtype=torch.int32)
    ids = torch.randint(0, vocab, (7,), generator=gen).to(torch.int32)
    turns = 10000.0 ** (-2.0 * torch.arange((width + 1) // 2, dtype=torch.float64) / width) / (2.0 * math.pi)
    out = torch.empty((7, width), device=DEV)
    K().embedding_sinusoids(out, table.to(DEV), ids.to(DEV), turns.to(DEV), positions.to(DEV), 1.5)
    angle = positions.double()[:, None] * 10000.0 ** (-2.0 * torch.arange((width + 1) // 2, dtype=torch.float64) / width)
    want = torch.stack([torch.sin(angle), torch.cos(angle)], dim=-1).flatten(1)[:, :width]
    assert torch.allclose(plain.position_vectors(512, width)[511], want[3], rtol=0.0, atol=1e-12)
    want = want + 1.5 * table.double()[ids.long()]
    assert float((out.cpu().double() - want).abs().max()) < 2e-6


# ----------------------------------------------------------------------------- query temperature and value mixing


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [dict(H=4, G=2, D=16, V=24, every=7, coef=0.5), dict(H=3, G=1, D=20, V=28, every=1, coef=1.5),
                                  dict(H=8, G=8, D=64, V=64, every=32, coef=-0.1), dict(H=2, G=2, D=9, V=5, every=1000, coef=0.3)])
def test_norms_temperature_and_mixed_values_reach_queries_and_cache(dtype, case):
    """From a position in the middle of a page on: queries normed and warmed, keys normed, values mixed with rows of
    another layer; the projected row keeps its own values; without norms the temperature still acts."""
    H, G, D, V, every, coef = (case[k] for k in ("H", "G", "D", "V", "every", "coef"))
    lib, gen = K(), torch.Generator().manual_seed(D)
    T, past, bs, eps, share = 37, 21, 16, 1e-5, 0.3
    width = H * D + G * D + G * V
    qkv = torch.randn((T, width + 3), generator=gen).to(dtype)     # rows wider than what they hold
    first = torch.randn((T, G * V + 2), generator=gen).to(dtype)
    wq, wk = (1.0 + 0.3 * torch.randn(D, generator=gen)).to(dtype), (1.0 + 0.3 * torch.randn(D, generator=gen)).to(dtype)
    pages = -(-(past + T) // bs)
    table = torch.randperm(pages + 1, generator=gen)[:pages].to(torch.int32)
    positions = torch.arange(past, past + T, dtype=torch.int32)
    rows = qkv.double()
    temp = plain.query_temperature(past + T, {"coef": coef, "every": every})[past:, None, None]
    q0, k0 = rows[:, :H * D].view(T, H, D), rows[:, H * D:(H + G) * D].view(T, G, D)
    v0 = rows[:, (H + G) * D:width].view(T, G, V)
    v = plain.mix_values(v0, first[:, :G * V].double().view(T, G, V), share)
    rel = 2e-6 if dtype == torch.float32 else 5e-3
    for normed in (True, False):
        q = (plain.over_rms(q0, eps) * wq.double() if normed else q0) * temp
        k = plain.over_rms(k0, eps) * wk.double() if normed else k0
        dev = qkv.to(DEV)
        kc = torch.zeros((pages + 1, G, bs, D), dtype=dtype, device=DEV)
        vc = torch.zeros((pages + 1, G, V, bs), dtype=dtype, device=DEV)
        lib.qk_norm_rotate_store(dev, H, G, D, V, wq.to(DEV) if normed else None, wk.to(DEV) if normed else None, eps, 0, False, None, 1.0,
                                 positions.to(DEV), torch.zeros(T, dtype=torch.int32, device=DEV), table.to(DEV)[None].contiguous(), bs, kc, vc,
                                 per_head=normed, temperature=(coef, every), mix=(first.to(DEV)[:, :G * V], share))
        close(dev[:, :H * D].view(T, H, D), q, rel, "queries")
        assert torch.equal(dev[:, (H + G) * D:].cpu(), qkv[:, (H + G) * D:])  # values (and what lies behind) as they were
        at = [(int(table[p // bs]), p % bs) for p in positions.tolist()]
        close(torch.stack([kc[b, :, o].cpu() for b, o in at]), k, rel, "cached keys")
        close(torch.stack([vc[b, :, :, o].cpu() for b, o in at]), v, rel, "cached values")


# ----------------------------------------------------------------------------- capped attention with a gate per head


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [dict(H=4, G=2, D=16, V=24, bs=8, cap=5.0), dict(H=8, G=2, D=64, V=64, bs=16, cap=20.0),
                                  dict(H=2, G=2, D=32, V=32, bs=32, cap=3.0), dict(H=6, G=1, D=128, V=128, bs=16, cap=30.0),
                                  dict(H=3, G=3, D=48, V=48, bs=16, cap=8.0), dict(H=4, G=4, D=96, V=96, bs=16, cap=0.0)])
def test_capped_scores_and_a_gate_per_head_whole_and_decoded(dtype, case):
    """A prompt of 300 and single tokens at its end, through every attention kernel that takes the shape.  For each query of
    a list one key is made to stand out: the first token, one on either side of a page's border, far back among hundreds,
    the query itself.  One head's gate is shut, another's wide open."""
    H, G, D, V, bs, cap = (case[k] for k in ("H", "G", "D", "V", "bs", "cap"))
    T, scale = 300, 0.25
    lib, gen = K(), torch.Generator().manual_seed(D + H)
    q, k = torch.randn((T, H, D), generator=gen) * 0.5, torch.randn((T, G, D), generator=gen) * 0.5
    v = torch.randn((T, G, V), generator=gen)
    loud = [(299, 0), (298, 2 * bs - 1), (297, 2 * bs), (296, 131), (295, 295), (40, 3)]
    for i, j in loud:
        k[j, 0] = 0.5 * torch.randn(D, generator=gen)
        q[i, 0] = k[j, 0] * 16.0 / (k[j, 0].norm() ** 2 * scale)   # score 16 before the cap, others of order one
    gate = torch.randn((T, H + 2), generator=gen)
    gate[:, 0], gate[:, H - 1] = 12.0, (-30.0 if H > 1 else 0.0)
    q, k, v, gate = (t.to(dtype) for t in (q, k, v, gate))
    want = plain.capped_softmax_attend(q.double(), k.double(), v.double(), scale, cap or None)
    if cap in (0.0, 20.0, 30.0):  # (a stronger cap leaves the loud key less than everything)
        assert float((want[299, 0] - v[0, 0].double()).abs().max()) < 0.2 * float(v[0, 0].double().abs().max())
    want = (want * plain.sigmoid(gate[:, :H].double())[:, :, None]).reshape(T, H * V)
    pages = -(-T // bs)
    table = torch.randperm(pages, generator=gen).to(torch.int32)
    kc, vc = torch.zeros((pages + 1, G, bs, D), dtype=dtype), torch.zeros((pages + 1, G, V, bs), dtype=dtype)
    for t in range(T):
        kc[table[t // bs], :, t % bs] = k[t]
        vc[table[t // bs], :, :, t % bs] = v[t]
    kc, vc, tab = kc.to(DEV), vc.to(DEV), table.to(DEV)[None].contiguous()
    qd, gd = q.to(DEV).view(T, H * D), gate.to(DEV)[:, :H]
    pos = torch.arange(T, dtype=torch.int32, device=DEV)
    rel = 2e-5 if dtype == torch.float32 else 2e-2
    out = torch.empty((T, H * V), dtype=dtype, device=DEV)
    lib.paged_attention_masked(out, qd, kc, vc, pos, torch.zeros(T, dtype=torch.int32, device=DEV), tab, H, G, D, V, scale, softcap=cap,
                               head_gate=gd)
    close(out, want, rel, f"any shape {case}")
    if not (dtype == torch.bfloat16 and V == D and lib.mfma_attention_supported(dtype, H, G, D, bs)):
        return
    from paged_attention_engine_amd.parts.attention import attend_paged, attention_work_lists
    for lens in ((T,), (T - 6,) + (1,) * 6, (100, 1, 57, 2, 140), (1,) * 3 + (T - 3,)):
        got, past = [], 0
        for n in lens:
            lists = attention_work_lists(step_shape((n,), (past,), bs))
            work = {name: on_device(flat, w) for name, (flat, w) in lists.items()}
            o = torch.zeros((n, H * V), dtype=dtype, device=DEV)
            attend_paged(o, qd[past:past + n], kc, vc, pos[past:past + n].contiguous(), None, tab, work, H, G, D, V, scale, 0, cap, None,
                         gd[past:past + n])
            got.append(o)
            past += n
        close(torch.cat(got), want, rel, f"matrix cores {case} {lens[:3]}")


# ----------------------------------------------------------------------------- matrix memory


def memory_plain(proj, logits, norm, H, D, V, cap, eps, dtype=torch.float64):
    T = proj.shape[0]
    p = proj.to(dtype)
    q = p[:, :H * D].view(T, H, D) * D ** -0.5
    k = p[:, H * D:2 * H * D].view(T, H, D)
    v = p[:, 2 * H * D:2 * H * D + H * V].view(T, H, V)
    gate = p[:, 2 * H * D + H * V:]
    z = logits.to(dtype)
    o = plain.matrix_memory_recurrence(q, k, v, plain.soft_cap(z[:, :H], cap), plain.log_sigmoid(plain.soft_cap(z[:, H:], cap)))
    return plain.over_rms(o, eps).reshape(T, H * V) * norm.to(dtype) * plain.sigmoid(gate)


def memory_step(lib, proj, logits, norm, H, D, V, cap, eps, lens, slots, state, top, gates_from=None):
    """`proj` [rows, 2HD + 2HV] = [q | k | v | gate] of the sequences `lens` one after the other."""
    from paged_attention_engine_amd.parts.delta import runs_and_chunks

    lists = runs_and_chunks(step_shape(lens, [0] * len(lens)), lib.matrix_memory_chunk(D))
    p = proj.to(DEV)
    out = torch.empty((proj.shape[0], H * V), dtype=proj.dtype, device=DEV)
    lib.matrix_memory_step(p, p[:, 2 * H * D + H * V:], None if gates_from else logits.to(DEV).contiguous(), out,
                           *(on_device(lists[name][0]) for name in ("serial", "chunks", "scans")),
                           torch.tensor(slots, dtype=torch.int32, device=DEV), state, top, norm.to(DEV), H, D, V, cap, eps, 1e-6,
                           gates_from=gates_from)
    return out


MEMORY_SHAPES = [(2, 16, 24), (3, 8, 40), (1, 64, 70), (4, 48, 32), (2, 72, 100), (1, 128, 128), (2, 130, 6), (2, 200, 64), (1, 260, 9),
                 (1, 520, 20), (3, 10, 14), (2, 30, 130)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", MEMORY_SHAPES)
def test_the_memory_whole_and_in_steps_in_used_slots(dtype, shape):
    """Every register grouping and both chunk lengths (key widths up to 64, 128, 256, and beyond, which take no chunks),
    widths that are no multiples of four or sixteen; gates beyond the cap on both sides; a sequence whole, token by token,
    and in portions that cross chunk edges in every way; beside another sequence; in slots that held other state."""
    H, D, V = shape
    lib, gen = K(), torch.Generator().manual_seed(D * 7 + V)
    T, eps, cap = 149, 1e-5, 6.0
    proj = (torch.randn((T, 2 * H * D + 2 * H * V), generator=gen) * 0.7).to(dtype)
    logits = torch.randn((T, 2 * H), generator=gen) * 3.0
    logits[T // 3] = 40.0 * cap
    logits[T // 2, :H] = -40.0 * cap
    logits[T // 2 + 9, H:] = -40.0 * cap
    norm = (1.0 + 0.2 * torch.randn((H * V,), generator=gen)).to(dtype)
    want = memory_plain(proj, logits, norm, H, D, V, cap, eps)
    rel = 2e-5 if dtype == torch.float32 else 6e-3
    state, top = torch.randn((4, H, V + 1, D), device=DEV), torch.randn((4, H), device=DEV)  # what other requests left

    def clear(slot):  # a slot is zeroed when a request takes it
        state[slot].zero_()
        top[slot].zero_()

    run = lambda rows, z, lens, slots: memory_step(lib, rows, z, norm, H, D, V, cap, eps, lens, slots, state, top)
    clear(1)
    close(run(proj, logits, (T,), [1]), want, rel, f"whole {shape}")
    whole_state, whole_top = state[1].clone(), top[1].clone()
    for cuts in ((1,) * T, (7, 2, 60, 1, 1, 33, 2, 17, 26), (17, 64, 3, 65), (5, 144), (128, 21)):
        clear(2)
        parts, at = [], 0
        for n in cuts:
            parts.append(run(proj[at:at + n], logits[at:at + n], (n,), [2]))
            at += n
        assert at == T
        close(torch.cat(parts), want, rel, f"steps {cuts[:3]} {shape}")
        close(state[2], whole_state, 2e-5, f"state after steps {shape}")
        assert float((top[2] - whole_top).abs().max()) < 1e-5
    for slot in (3, 0, 2):
        clear(slot)
    both, zs = torch.cat([proj[:9], proj[:T], proj[:1]]), torch.cat([logits[:9], logits[:T], logits[:1]])
    got = run(both, zs, (9, T, 1), [3, 0, 2])
    close(got[9:9 + T], want, rel, f"beside others {shape}")
    close(got[:9], want[:9], rel, f"the short run {shape}")
    close(got[9 + T:], want[:1], rel, f"the single token {shape}")
    close(state[0], whole_state, 2e-5, f"state beside others {shape}")


def memory_case(T, H, D, V, seed=1):
    gen = torch.Generator().manual_seed(seed)
    return gen, torch.randn((T, 2 * H * D + 2 * H * V), generator=gen) * 0.5, torch.zeros((T, 2 * H))


def fresh(H, D, V):
    return torch.zeros((1, H, V + 1, D), device=DEV), torch.zeros((1, H), device=DEV)


@pytest.mark.parametrize("marks", [(40, 299), (63, 64), (62, 63), (127, 128), (0, 191), (1023, 1024), (5, 1100)])
def test_the_memory_keeps_what_it_was_told_to(marks):
    """A forget gate wide open and one input gate far above the others: the read-out is that token's value, many tokens
    later, and across the edges of chunks and of what the gates' kernel takes at a time."""
    written, read = marks
    H, D, V, T, cap = 1, 32, 16, read + 1, 20.0
    _, proj, logits = memory_case(T, H, D, V)
    logits[:, 0], logits[:, 1] = -15.0, 15.0
    logits[written, 0] = 15.0
    proj[read, :D] = proj[written, D:2 * D] * 4  # the last query asks for the written key
    want = memory_plain(proj, logits, torch.ones(V), H, D, V, cap, 1e-6)
    # where n . q nearly cancels, the division blows rounding up: a token is allowed what float32 does to the plain recurrence
    rounding = (memory_plain(proj, logits, torch.ones(V), H, D, V, cap, 1e-6, torch.float32).double() - want).abs().amax(1)
    bound = 2e-5 * float(want.abs().max()) + 4.0 * rounding
    assert float((rounding > 1e-4).double().mean()) < 0.01 and rounding[read] < 1e-5
    for lens in ((T,), (written + 1, read - written)):
        state, top = fresh(H, D, V)
        at, parts = 0, []
        for n in lens:
            parts.append(memory_step(K(), proj[at:at + n], logits[at:at + n], torch.ones(V), H, D, V, cap, 1e-6, (n,), [0], state, top))
            at += n
        got = torch.cat(parts)
        assert bool(((got.cpu().double() - want).abs().amax(1) <= bound).all()), f"recall {marks} {lens}"
        value = proj[written, 2 * D:2 * D + V].double()
        direction = plain.over_rms(value[None], 1e-6)[0] * plain.sigmoid(proj[read, 2 * D + V:].double())
        assert float((got[read].cpu().double() - direction).abs().max()) < 0.05 * float(direction.abs().max())


def test_a_long_fade_does_not_blur_what_follows_it():
    """Forget gates shut for half a chunk (the logarithm of what is kept falls by hundreds) and wide open after: the
    differences of those logarithms that weigh the later tokens must be as exact as if nothing had come before."""
    H, D, V, T, cap = 2, 16, 12, 64, 15.0
    gen, proj, logits = memory_case(T, H, D, V, seed=5)
    logits[:32, H:] = -200.0
    logits[32:, H:] = 60.0
    logits[:, :H] = torch.randn((T, H), generator=gen)
    want = memory_plain(proj, logits, torch.ones(H * V), H, D, V, cap, 1e-6)
    state, top = fresh(H, D, V)
    got = memory_step(K(), proj, logits, torch.ones(H * V), H, D, V, cap, 1e-6, (T,), [0], state, top)
    close(got, want, 5e-6, "after the fade")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden", [64, 90, 1536])
def test_gates_formed_from_the_mixers_input(dtype, hidden):
    """Short runs form the gates' sums inside the kernel that uses them: the same read-outs as from the product."""
    H, D, V, cap, lens = 3, 24, 20, 7.0, (1, 16, 5, 1)
    gen, proj, _ = memory_case(sum(lens), H, D, V, seed=hidden)
    proj = proj.to(dtype)
    x = torch.randn((sum(lens), hidden), generator=gen).to(dtype)
    w = (torch.randn((2 * H, hidden), generator=gen) * 2.0 / hidden ** 0.5).to(dtype)
    b = torch.randn(2 * H, generator=gen)
    logits = (x.double() @ w.double().T + b.double()).float()
    rel = 1e-5 if dtype == torch.float32 else 5e-3
    state, top = torch.zeros((4, H, V + 1, D), device=DEV), torch.zeros((4, H), device=DEV)
    got = memory_step(K(), proj, None, torch.ones(H * V), H, D, V, cap, 1e-5, lens, [2, 0, 3, 1], state, top,
                      gates_from=(x.to(DEV), w.to(DEV), b.to(DEV)))
    at = 0
    for n in lens:
        want = memory_plain(proj[at:at + n], logits[at:at + n], torch.ones(H * V), H, D, V, cap, 1e-5)
        close(got[at:at + n], want, rel, f"run of {n}")
        at += n


# ----------------------------------------------------------------------------- feed-forwards


class Context:
    sink = None

    def __init__(self, takes_bias_terms=False):
        self.takes_bias_terms = takes_bias_terms


def part_of(spec, weights, dtype):
    from paged_attention_engine_amd.parts import FEED_FORWARDS, build_part

    part = build_part(FEED_FORWARDS, "feed-forward", spec, dtype, DEV)
    assert {name: tuple(shape) for name, shape in part.tensors("f.").items()} == {name: tuple(t.shape) for name, t in weights.items()}
    part.bind("f.", weights)
    return part


def total(y):
    """A branch's output, whatever form it came in, as one tensor."""
    if isinstance(y, list):
        return sum(factor * total(term) for term, factor in y)
    return y.double().sum(0) if y.dim() == 3 else y.double()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [(64, 88), (90, 50), (128, 256), (72, 1032)])
def test_dense_with_biases_and_the_square_of_relu(dtype, case):
    """Few rows (the bias and the activation in the product's epilogue) and many (in the activation's own kernel)."""
    from paged_attention_engine_amd.config.model_config import FeedForwardSpec

    H, F = case
    gen = torch.Generator().manual_seed(F)
    draw = lambda *shape: torch.randn(shape, generator=gen)
    weights = {"f.up": (draw(F, H) * H ** -0.5).to(torch.bfloat16), "f.up.b": draw(F).to(torch.bfloat16),
               "f.down": (draw(H, F) * F ** -0.5).to(torch.bfloat16), "f.down.b": draw(H).to(torch.bfloat16)}
    part = part_of(FeedForwardSpec(kind="dense", hidden_size=H, intermediate_size=F, activation="relu2", up_name="up", down_name="down",
                                   weight_suffix="", bias=True, bias_suffix=".b"), weights, dtype)
    for T in (1, 5, 17, 64, 65, 200):
        x = draw(T, H).to(dtype)
        want = plain.dense(weights, "f.", x.double(), torch.float64)
        for takes in (False, True):  # the second product's bias inside the product, or left to the norm that follows
            y = part.forward(Context(takes), x.to(DEV))
            assert isinstance(y, list) == (takes and dtype == torch.bfloat16)
            close(total(y), want, 1e-5 if dtype == torch.float32 else 2e-2, f"{T} rows {case}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H", [48, 90, 1536])
def test_a_product_and_its_bias_join_through_offset_norms(dtype, H):
    """x <- x + (1 + w) * normed(parts + bias), and the norm before the next sublayer, whose weight is stored around zero too."""
    gen = torch.Generator().manual_seed(H)
    T, eps = 9, 1e-4
    x, parts = torch.randn((T, H), generator=gen), torch.randn((3, T, H), generator=gen)
    bias = torch.randn(H, generator=gen).to(dtype)
    w_out, w_next = torch.randn(H, generator=gen) * 0.3, torch.randn(H, generator=gen) * 0.3
    y = parts.double().sum(0) + bias.double()
    new = x.double() + plain.offset_norm(y, w_out.double(), eps)
    residual, normed = x.to(DEV), torch.empty((T, H), dtype=dtype, device=DEV)
    K().norm_join(residual, [(parts.to(DEV), 1.0), (bias.to(DEV), 1.0)], (1 + w_out).to(DEV), eps, (1 + w_next).to(DEV), eps, normed)
    close(residual, new, 2e-6, "the new stream")
    close(normed, plain.offset_norm(new, w_next.double(), eps), 1e-5 if dtype == torch.float32 else 1e-2, "the next norm")


@pytest.mark.parametrize("case", [dict(E=6, top=2), dict(E=9, top=1), dict(E=4, top=4), dict(E=64, top=6), dict(E=200, top=8), dict(E=1, top=1)])
@pytest.mark.parametrize("pieces", [0, 1, 3])
def test_routing_weighs_the_chosen_logits_alone(case, pieces):
    """Also with logits far too large to exponentiate, and far apart; the shared pieces carry their own sigmoid."""
    E, top = case["E"], case["top"]
    for factor, shift in ((2.0, 0.0), (1.0, 5000.0), (300.0, 0.0)):
        gen = torch.Generator().manual_seed(E)
        z = torch.randn((300, E + (1 if pieces else 0)), generator=gen) * factor + shift
        if pieces:
            z[:, E] = torch.randn(300, generator=gen) * 3.0
        want_chosen, want_weights = plain.route(z[:, :E].double(), top)
        chosen, weights = K().moe_route(z.to(DEV), 1, 1, top, 1.0, among_chosen=True, shared_pieces=pieces)
        assert chosen.shape == weights.shape == (300, top + pieces)
        assert torch.equal(chosen[:, :top].cpu().long(), want_chosen)  # in order of falling logits
        assert float((weights[:, :top].cpu().double() - want_weights).abs().max()) < 1e-6
        for p in range(pieces):
            assert torch.equal(chosen[:, top + p].cpu(), torch.full((300,), E + p, dtype=torch.int32))
            assert float((weights[:, top + p].cpu().double() - plain.sigmoid(z[:, E].double())).abs().max()) < 1e-6


def test_of_equal_logits_the_lower_index_is_chosen():
    z = torch.tensor([[1.0, 2.0, 2.0, 2.0, 0.0], [0.0, 0.0, 0.0, 0.0, 0.0]])
    chosen, weights = K().moe_route(z.to(DEV), 1, 1, 2, 1.0, among_chosen=True)
    assert chosen.cpu().tolist() == [[1, 2], [0, 1]] and weights.cpu().tolist() == [[0.5, 0.5], [0.5, 0.5]]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [dict(H=64, F=24, E=5, top=2, shared=40), dict(H=64, F=32, E=4, top=2, shared=32), dict(H=90, F=14, E=3, top=3, shared=5),
                                  dict(H=96, F=64, E=6, top=1, shared=160), dict(H=64, F=32, E=7, top=3, shared=None)])
@pytest.mark.parametrize("T", [1, 9, 130, 700])
def test_routed_experts_with_a_shared_one(dtype, case, T):
    """The whole feed-forward against the plain one on its own choices, which must be the plain ones where they are clear:
    a shared expert narrower than the routed ones, as wide, and of several pieces, in every size class of the kernels."""
    from paged_attention_engine_amd.config.model_config import ExpertsSpec, SharedExpertSpec

    H, F, E, top, shared = (case[k] for k in ("H", "F", "E", "top", "shared"))
    gen = torch.Generator().manual_seed(H + F)
    draw = lambda *shape: (torch.randn(shape, generator=gen) * shape[-1] ** -0.5).to(torch.bfloat16)
    weights = {"f.router": draw(E, H), "f.router.b": (torch.randn(E, generator=gen) * 0.5).to(torch.bfloat16)}
    sizes = [(f"e{e}.", F) for e in range(E)] + ([("shared.", shared)] if shared else [])
    for name, width in sizes:
        weights.update({f"f.{name}gate": draw(width, H), f"f.{name}up": draw(width, H), f"f.{name}down": draw(H, width)})
    if shared:
        weights["f.shared.sg"] = draw(1, H)
    spec = ExpertsSpec(hidden_size=H, intermediate_size=F, num_experts=E, top=top, router_bias_name="router.b", weights_over="chosen",
                       shared=SharedExpertSpec(shared) if shared else None)
    part = part_of(spec, weights, dtype)
    taken = []
    part.routing_tap = lambda chosen, w: taken.append(chosen.cpu().long())
    x = torch.randn((T, H), generator=gen).to(dtype)
    got = total(part.forward(Context(), x.to(DEV)))
    mlp = {"router": {"experts": E, "top": top}, "shared": {"ff": shared} if shared else None}
    margins = []
    want = plain.mixture(weights, "f.", mlp, x.double(), torch.float64, margins, forced=taken[0])
    free, _ = plain.route(x.double() @ weights["f.router"].double().T + weights["f.router.b"].double(), top)
    clear = margins[0] > 1e-4
    assert torch.equal(taken[0][clear].sort(-1).values, free[clear].sort(-1).values) and clear.float().mean() > 0.9
    close(got, want, 1e-5 if dtype == torch.float32 else 2e-2, f"{case} {T} rows")
