"""The Getodra model through the engine's step function, cache and kernels against the plain
implementation (tests/plain/getodra_plain.py, float64 on the same weights).

Per model and precision one replayer runs the same requests whole, decoded token by token from the
first token on, in portions of several sizes down to two tokens, and mixed: unequal requests side by
side in a pool and in state slots so small that pages and slots are given back and used again.  Every
logit is compared with the plain one.  Greedy generation goes through the engine's own entry point and
scheduler, through `bin/trace_run` as a program, and through the command line.
"""

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import getodra_models as M
from tests import helpers
from tests.plain import getodra_plain as plain

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LENGTHS = (150, 37, 90, 1)
PORTIONS = (7, 2, 5, 3, 2, 11, 4, 2, 9, 17, 33)
DTYPES = ("float32", "bfloat16")


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("getodra")
    return {name: M.make_folder(tmp, name) for name in M.CONFIGS}


_PLAIN, _WEIGHTS, _ROUNDING = {}, {}, {}


def weights_of(folders, name):
    if name not in _WEIGHTS:
        _WEIGHTS[name] = M.read_folder(folders[name])
    return _WEIGHTS[name]


def plain_logits(folders, name, tokens):
    key = (name, tuple(tokens))
    if key not in _PLAIN:
        cfg, weights = weights_of(folders, name)
        _PLAIN[key] = plain.forward(weights, cfg, tokens, torch.float64, angle_dtype=torch.float32)
    return _PLAIN[key]


def rounding_alone(folders, name, tokens):
    """The largest error of the plain implementation when its products' operands and results are rounded to
    bfloat16 and nothing else changes."""
    key = (name, tuple(tokens))
    if key not in _ROUNDING:
        cfg, weights = weights_of(folders, name)
        want = plain_logits(folders, name, tokens)
        worst = 0.0
        plain.STORAGE = torch.bfloat16
        try:
            for trial in range(2):  # the products' sums as they are, and in another order of adding
                plain.JITTER = (torch.Generator().manual_seed(trial), 3e-4) if trial else None
                got = plain.forward(weights, cfg, tokens, torch.float64, angle_dtype=torch.float32)
                worst = max(worst, float((got - want).abs().max()))
        finally:
            plain.STORAGE = plain.JITTER = None
        _ROUNDING[key] = worst
    return _ROUNDING[key]


def check(got, folders, name, tokens, dtype, what, rows=slice(None)):
    """float32: a few hundred roundings relative to the largest logit.  bfloat16: the engine may be off by
    three times what rounding alone does to the plain implementation on the same tokens, plus a unit in
    the last place of the largest logit."""
    want = plain_logits(folders, name, tokens)[rows]
    got = torch.as_tensor(got).double()
    worst = float((got - want).abs().max())
    bound = 1e-4 * float(want.abs().max())
    if dtype == "bfloat16":
        bound = 3.0 * rounding_alone(folders, name, tokens) + helpers.bf16_ulp(want)
    assert worst <= bound, f"{what}: worst logit error {worst:.3e} > {bound:.3e}"


def replayer(folders, name, dtype, max_tokens, max_live=4, block_size=16):
    from paged_attention_engine_amd.engine.trace import TraceReplayer

    return TraceReplayer(folders[name], dtype, max_tokens, block_size, max_live)


def alone(rp, rid, tokens, cuts):
    """Feed `tokens` as one request in portions of the sizes `cuts` (cycled): [T, vocab]."""
    rows, p, i = [], 0, 0
    while p < len(tokens):
        n = min(cuts[i % len(cuts)], len(tokens) - p)
        i += 1
        out = rp.step({"step": 0, "entries": [{"id": rid, "tokens": tokens[p:p + n], "want": list(range(n))}],
                       "end": [rid] if p + n == len(tokens) else []})
        rows.append(torch.from_numpy(out.copy()))
        p += n
    return torch.cat(rows)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(M.CONFIGS))
def test_whole_decoded_and_in_portions(folders, name, dtype):
    """A prompt whole, token by token from its first token on (which is prefill against decoding, and a
    long decode), and in portions of changing sizes: all against the plain logits, and in float32 the
    ways against each other to a few roundings.  150 tokens cross the edges of pages, of the recurrence's chunks
    and of the convolutions' tiles."""
    rp = replayer(folders, name, dtype, 256)
    for length in LENGTHS[:3]:
        tokens = M.tokens_for(name, length)
        ways = {"whole": (length,), "token by token": (1,), "portions": PORTIONS, "other portions": PORTIONS[4:] + PORTIONS[:4],
                "portions of two": (2,), "a long portion in the middle": (5, 85, 1, 1, 2)}
        outs = {}
        for way, cuts in ways.items():
            outs[way] = alone(rp, way, tokens, cuts)
            check(outs[way], folders, name, tokens, dtype, f"{name} {dtype} {way} {length}")
        if dtype == "float32":
            top = float(outs["whole"].abs().max())
            for way, out in outs.items():
                assert float((outs["whole"] - out).abs().max()) <= 2e-5 * top, f"{name} {way} against whole"
    assert rp.cache.slots.num_free == 4 and all(g.allocator.num_free == g.allocator.num_blocks for g in rp.cache.groups)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(M.CONFIGS))
def test_the_first_tokens_of_a_sequence(folders, name, dtype):
    """One token to seven, each as a request of its own: the first positions' rows, the zeros a convolution sees before
    the sequence (fewer tokens than taps), the state's start, a softmax of one key."""
    rp = replayer(folders, name, dtype, 64)
    for length in range(1, 8):
        tokens = M.tokens_for(name, length, salt=7)
        for way, cuts in (("whole", (length,)), ("one by one", (1,)), ("by two", (2,))):
            check(alone(rp, way, tokens, cuts), folders, name, tokens, dtype, f"{name} first {length} {way}")


def mixed_schedule(lengths):
    """Steps of (request index, count): requests arrive staggered, run a portion a step and then single
    tokens beside the others' portions; at most four are live; every request runs twice."""
    order = [i for _ in range(2) for i in range(len(lengths))]
    steps, live, arrivals = [], {}, list(enumerate(order))
    tick = 0
    while arrivals or live:
        if arrivals and len(live) < 4 and tick % 2 == 0:
            rid, which = arrivals.pop(0)
            live[rid] = [which, 0]
        step = []
        for rid, (which, at) in list(live.items()):
            remaining = lengths[which] - at
            tail = min(12, lengths[which] // 2)
            n = 1 if remaining <= tail else min(PORTIONS[(tick + rid) % len(PORTIONS)], remaining - tail)
            if (tick + rid) % 5 == 4 and remaining > 1:
                continue  # a request is left out of a step and goes on later
            step.append((rid, which, at, n))
            live[rid][1] = at + n
            if at + n == lengths[which]:
                del live[rid]
        if step:
            steps.append(step)
        tick += 1
    return steps


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(M.CONFIGS))
def test_unequal_requests_side_by_side_with_pages_and_slots_used_again(folders, name, dtype):
    tokens = [M.tokens_for(name, n) for n in LENGTHS]
    steps = mixed_schedule(LENGTHS)
    # the pool holds what the four longest live requests need and no more, so pages are used again
    rp = replayer(folders, name, dtype, sum(-(-n // 64) * 64 for n in LENGTHS))
    rows_of = {}
    for step in steps:
        record = {"step": 0, "entries": [], "end": []}
        for rid, which, at, n in step:
            record["entries"].append({"id": f"r{rid}", "tokens": tokens[which][at:at + n], "want": list(range(n))})
            if at + n == LENGTHS[which]:
                record["end"].append(f"r{rid}")
        out, row = torch.from_numpy(rp.step(record).copy()), 0
        for rid, which, at, n in step:
            rows_of.setdefault((rid, which), []).append(out[row:row + n])
            row += n
    assert len(steps) > 30 and max(len(s) for s in steps) == 4
    for (rid, which), rows in rows_of.items():
        check(torch.cat(rows), folders, name, tokens[which], dtype, f"{name} {dtype} request {rid}")
    assert rp.cache.slots.num_free == 4
    if rp.runner.use_graphs and rp.runner.graph_max_rows != 0:
        assert rp.runner.graph_replays > 0  # steps of single tokens ran as recorded graphs


@pytest.mark.parametrize("name", ["P", "R"])
def test_a_slot_that_held_another_request_starts_from_zero(folders, name):
    """One state slot: every request takes the slot the one before gave back (state matrices and the convolutions'
    inputs of every stop), and must not see any of it."""
    rp = replayer(folders, name, "float32", 128, max_live=1)
    for length in (37, 90, 2, 37):
        tokens = M.tokens_for(name, length)
        check(alone(rp, "s", tokens, (5, 1, 1, 40)), folders, name, tokens, "float32", f"{name} in a used slot, {length}")


def test_long_decoding(folders):
    """Two requests decode 180 tokens side by side in recorded steps after prompts of 3 and 70 tokens."""
    tokens = [M.tokens_for("R", 183, salt=1), M.tokens_for("R", 250, salt=2)]
    for dtype in DTYPES:
        rp = replayer(folders, "R", dtype, 512)
        at, rows = [3, 70], [[], []]
        first = rp.step({"step": 0, "entries": [{"id": f"r{i}", "tokens": tokens[i][:at[i]], "want": list(range(at[i]))} for i in (0, 1)]})
        rows[0].append(torch.from_numpy(first[:3].copy()))
        rows[1].append(torch.from_numpy(first[3:].copy()))
        for step in range(180):
            out = rp.step({"step": 0, "entries": [{"id": f"r{i}", "tokens": [tokens[i][at[i] + step]], "want": [0]} for i in (0, 1)]})
            for i in (0, 1):
                rows[i].append(torch.from_numpy(out[i:i + 1].copy()))
        for i in (0, 1):
            check(torch.cat(rows[i]), folders, "R", tokens[i], dtype, f"long decoding {dtype} {i}")
        assert rp.runner.graph_replays == 180


def test_the_stream_after_every_layer(folders):
    """The float32 stream after each layer against the plain one; a layer that borrows tensors is seen like any other."""
    from paged_attention_engine_amd.engine.step import StepRunner

    for name in ("P", "Q"):
        rp = replayer(folders, name, "float32", 64)
        rp.runner = StepRunner(rp.model, rp.cache, use_graphs=False)
        seen = []
        rp.model.residual_tap = lambda index, stream: seen.append(stream.residual.clone().cpu().double())
        tokens = M.tokens_for(name, 37)
        alone(rp, "t", tokens, (37,))
        cfg, weights = weights_of(folders, name)
        taps = []
        plain.forward(weights, cfg, tokens, torch.float64, taps=taps, angle_dtype=torch.float32)
        assert len(seen) == len(taps) == len(cfg["layers"])
        for i, (got, want) in enumerate(zip(seen, taps)):
            assert float((got - want).abs().max()) <= 2e-5 * float(want.abs().max()), f"{name} layer {i}"


@pytest.mark.parametrize("name, dtype", [("P", "float32"), ("R", "bfloat16")])
def test_recorded_steps_give_the_eager_steps_logits(folders, name, dtype):
    """Steps of single tokens replay as HIP graphs; the same steps launched kernel by kernel give the same bits."""
    from paged_attention_engine_amd.engine.step import StepRunner

    tokens = M.tokens_for(name, 60)
    outs = []
    for graphs in (True, False):
        rp = replayer(folders, name, dtype, 128)
        rp.runner = StepRunner(rp.model, rp.cache, use_graphs=graphs)
        outs.append(alone(rp, "a", tokens, (20,) + (1,) * 40))
        if graphs:
            assert rp.runner.graph_replays >= 39
    assert torch.equal(outs[0], outs[1])


@pytest.mark.parametrize("name", ["P", "R"])
def test_greedy_generation_through_the_entry_point(folders, name):
    import paged_attention_engine_amd as pae

    cfg, weights = weights_of(folders, name)
    prompt = M.tokens_for(name, 21, salt=3)
    want_tokens, want_logits = plain.greedy_generate(weights, cfg, prompt, 12, torch.float64)
    assert len(set(want_tokens)) > 2
    engine = pae.Engine(folders[name], dtype="float32", block_size=16, num_blocks=8, max_num_seqs=2)
    got = engine.generate(prompt, 12)
    assert list(got.token_ids) == want_tokens
    assert float((got.step_logits.cpu().double() - want_logits).abs().max()) <= 1e-4 * float(want_logits.abs().max())
    # bfloat16: the same entry point; its tokens agree until two plain logits nearly tie
    engine = pae.Engine(folders[name], dtype="bfloat16", block_size=16, num_blocks=8, max_num_seqs=2)
    got = list(engine.generate(prompt, 12).token_ids)
    assert len(got) == 12
    same = next((i for i in range(12) if got[i] != want_tokens[i]), 12)
    if same < 12:
        top2 = want_logits[same].topk(2).values
        bound = 3.0 * rounding_alone(folders, name, prompt + want_tokens[:same]) + helpers.bf16_ulp(want_logits)
        assert float(top2[0] - top2[1]) <= 2.0 * bound


def test_requests_through_the_scheduler_with_few_pages(folders):
    """Several requests through the scheduler in a pool that forces waiting and portions; every request's
    tokens are those it generates alone."""
    import paged_attention_engine_amd as pae

    prompts = [M.tokens_for("P", n, salt=9) for n in (33, 5, 70, 18, 41)]
    single = []
    for prompt in prompts:
        engine = pae.Engine(folders["P"], dtype="float32", block_size=16, num_blocks=16, max_num_seqs=1)
        single.append(list(engine.generate(prompt, 10).token_ids))
    engine = pae.Engine(folders["P"], dtype="float32", block_size=16, num_blocks=14, max_num_seqs=3,
                        max_num_batched_tokens=24)
    for i, prompt in enumerate(prompts):
        assert engine.add_request(pae.Request(f"r{i}", tuple(prompt), max_new_tokens=10))
    done = engine.run_to_completion()
    assert [list(done[f"r{i}"]) for i in range(len(prompts))] == single


@pytest.mark.parametrize("dtype", DTYPES)
def test_recorded_steps_padded_beyond_eight_requests(folders, dtype):
    """Ten requests decode side by side: the recorded step is padded to twelve rows, whose padding rows share one page and
    one state slot that no request holds.  Every logit is the plain one."""
    rp = replayer(folders, "R", dtype, 10 * 64, max_live=10)
    tokens = [M.tokens_for("R", 30 + i, salt=i) for i in range(10)]
    rp.step({"step": 0, "entries": [{"id": f"r{i}", "tokens": t[:-12], "want": []} for i, t in enumerate(tokens)]})
    rows = [[] for _ in tokens]
    for back in range(12, 0, -1):
        out = rp.step({"step": 0, "entries": [{"id": f"r{i}", "tokens": [t[len(t) - back]], "want": [0]} for i, t in enumerate(tokens)]})
        for i in range(10):
            rows[i].append(torch.from_numpy(out[i:i + 1].copy()))
    assert rp.runner.graph_replays == 12
    for i, t in enumerate(tokens):
        check(torch.cat(rows[i]), folders, "R", t, dtype, f"ten at once {dtype} {i}", slice(len(t) - 12, None))


def test_a_request_that_would_pass_the_last_position_is_refused(folders):
    """The model has a row for every position up to max_positions and none beyond: the admission guard says no."""
    import paged_attention_engine_amd as pae

    engine = pae.Engine(folders["S"], dtype="float32", block_size=16, num_blocks=32, max_num_seqs=2)
    limit = M.S["max_positions"]
    assert not engine.add_request(pae.Request("long", tuple(M.tokens_for("S", limit - 3)), max_new_tokens=10))
    assert engine.add_request(pae.Request("fits", tuple(M.tokens_for("S", limit - 12)), max_new_tokens=10))


def test_the_program_replays_a_trace(folders, tmp_path):
    """bin/trace_run as a program: steps on standard input, logits in files, `done` lines."""
    tokens = M.tokens_for("Q", 37)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": tokens[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": tokens[20:22], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": tokens[22:], "want": [14]}], "end": ["a"]}]
    out = tmp_path / "logits"
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders["Q"], "--dtype",
                           "float32", "--out", str(out), "--max-tokens", "64"],
                          input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [line for line in proc.stdout.splitlines() if line.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert not (out / "1.f32").exists()
    first = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(2, -1))
    last = torch.from_numpy(np.fromfile(out / "2.f32", dtype="<f4").reshape(1, -1))
    check(first, folders, "Q", tokens, "float32", "trace_run step 0", [0, 19])
    check(last, folders, "Q", tokens, "float32", "trace_run step 2", [36])


def test_the_command_line_generates_and_samples(folders):
    """`python -m paged_attention_engine_amd` on a model folder: greedy tokens of two prompts are the plain ones; with a
    temperature the same seed gives the same tokens twice and another seed gives others."""
    cfg, weights = weights_of(folders, "Q")
    prompts = [M.tokens_for("Q", 19, salt=5), M.tokens_for("Q", 7, salt=6)]
    want = [plain.greedy_generate(weights, cfg, p, 6, torch.float64)[0] for p in prompts]

    def run(*extra):
        cmd = [sys.executable, "-m", "paged_attention_engine_amd", "--model", folders["Q"], "--dtype", "float32", "--max-new-tokens", "6",
               "--num-blocks", "16", "--max-num-seqs", "2"]
        for p in prompts:
            cmd += ["--prompt-ids", ",".join(map(str, p))]
        proc = subprocess.run(cmd + list(extra), capture_output=True, text=True, timeout=600, cwd=ROOT)
        assert proc.returncode == 0, proc.stderr[-2000:]
        lines = [json.loads(line) for line in proc.stdout.splitlines() if line.startswith("{")]
        return [line["token_ids"] for line in lines]

    assert run() == want
    first = run("--temperature", "0.9", "--sample-seed", "3")
    assert first == run("--temperature", "0.9", "--sample-seed", "3")
    assert first != run("--temperature", "0.9", "--sample-seed", "4") and first != want
