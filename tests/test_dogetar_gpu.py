"""Dogetar through the engine (loader, cache and state pools, scheduler, captured decode graphs) against
``oracle/dogetar_ref.py``: whole prompts, portions, decoding, unequal batches, blocks and slots used again, greedy
generation.  float32 has to agree to rounding; in bfloat16 every position has a limit of its own, a multiple of what
rounding the activations alone does to it, and a few positions whose choice of experts is a close call may differ."""
import json
import subprocess
import sys

import numpy as np
import pytest
import torch

from infer_amd.sampling_params import SamplingParams
from infer_amd.trace import TraceReplay
from oracle import dogetar_ref as ref
from tests import dogetar_helpers as dh, merilorn_helpers as mh
from tests.test_merilorn_gpu import BF16, DT, F32, engine, feed, greedy_is_right

pytestmark = pytest.mark.gpu

CONFIGS = {
    "mixed-layers": dh.small_config,
    # sizes that are multiples of nothing, one head, one group, no loop, no second embedding
    "odd": lambda: dh.make_config([dh.parallel(1, 1, 10, 7, 19, ssm=(1, 6, 5, 1, 3, 2), mlp=dh.moe(9, 3, 0, 1, 1, 1, 1.0, None)),
                                   dh.chunked(1, 1, 9, 11, 21, rot_dims=6, mlp=dh.dense(30)),
                                   dh.windowed(3, 1, 13, 5, 23, rot_dims=10, scaling=None)], width=50, vocab=77, cap=40.0, bigram=None),
    # heads of the sizes of published models: every layer on the matrix pipe
    "wide": lambda: dh.make_config([dh.windowed(8, 2, 64, 64, 70, 0.1, 32, mlp=dh.moe(64, 8, 0, 2, 4, 2, 2.0, 64)),
                                    dh.chunked(4, 2, 32, 64, 96, 0.2, rot_dims=32, mlp=dh.dense(128)),
                                    dh.parallel(4, 4, 64, 64, 80, 0.1, ssm=(4, 64, 64, 2, 4, 2))], width=128, vocab=100, loop=(0, 3, 2)),
    # masks of one token and longer than any prompt; a loop of one pass; experts of one kind only
    "edges": lambda: dh.make_config([dh.windowed(size=1, mlp=dh.moe(16, 2, 2, 3, 1, 1)), dh.chunked(size=1), dh.windowed(size=5000),
                                     dh.parallel(size=5000, ssm=(2, 136, 128, 1, 4, 1)), dh.chunked(4, 4, 16, 136, 5000)], loop=(4, 5, 1)),
    "state-space": lambda: dh.make_config([dh.parallel(ssm=(8, 8, 256, 8, 2, 8)), dh.parallel(ssm=(2, 32, 40, 2, 1, 4), mlp=dh.dense())],
                                          loop=(1, 2, 3), eps=1e-2),
}


def check(got, want, limit):
    assert np.isfinite(got).all()
    over = mh.row_errors(got, want) / limit
    if limit.max() <= F32:
        assert over.max() <= 1.0, (np.argmax(over), over.max())
    else:
        assert (over > 1.0).mean() <= 0.04, (np.flatnonzero(over > 1.0)[:10], over.max())


class Model:
    def __init__(self, folder, name, config=None, weights=None):
        self.config = config or CONFIGS[name]()
        self.weights = weights or dh.make_weights(self.config, seed=sum(map(ord, name)))
        self.folder = mh.save_model(folder, self.config, self.weights)

    def logits(self, toks):
        return ref.forward(self.config, self.weights, toks)[0]

    def limits(self, toks, dtype):
        """The wanted logits and the limit of every position's error."""
        want = self.logits(toks)
        if dtype == "float32":
            return want, np.full(len(toks), F32)
        rounded = ref.forward(self.config, self.weights, toks, cast=mh.bf16)[0]
        return want, np.maximum(BF16, 3 * mh.row_errors(rounded, want))


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = Model(tmp_path_factory.mktemp(name), name)
        return made[name]
    return get


def tensors(storage):
    """Every tensor of a runner's cache, whatever it is nested in."""
    if isinstance(storage, torch.Tensor):
        return [storage]
    return [t for part in (storage.values() if isinstance(storage, dict) else storage) for t in tensors(part)]


@DT
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_decode_and_portions(gpu, models, name, dtype):
    m = models(name)
    n = 150
    toks = mh.tokens(n, m.config, 1)
    want, limit = m.limits(toks, dtype)
    trace = TraceReplay(m.folder, dtype, 192)
    cuts = [[n], [n - 20] + [1] * 20, [2] * 20 + [64, 33, 1, 1, 3, 8], [1] * n, [66, 65, 2, 17], [1, 70, 1, 63, 15], [31, 32, 33, 54]]
    for i, c in enumerate(cuts):
        check(feed(trace, f"r{i}", toks, c), want, limit)
    sched = trace.engine.scheduler
    assert sched.block_manager.num_free_blocks == 3 and sched.slots.num_free == 4


@DT
def test_unequal_requests_in_one_batch_and_pages_and_slots_used_again(gpu, models, dtype):
    m = models("mixed-layers")
    trace = TraceReplay(m.folder, dtype, 640)
    rng = np.random.default_rng(4)
    live, done, made, results = {}, 0, 0, []
    while done < 10:
        while len(live) < 4 and made < 10:
            n = [130, 3, 70, 1, 129, 64, 90, 2, 65, 100][made]
            toks = mh.tokens(n, m.config, 100 + made)
            live[f"q{made}"] = [toks, 0, *m.limits(toks, dtype)]
            made += 1
        entries, end, expect, limit = [], [], [], []
        for name in sorted(live, key=lambda _: rng.random()):
            toks, lo, want, lim = live[name]
            if rng.random() < 0.2:
                continue                               # left out of this step
            c = min(int(rng.choice([1, 1, 2, 3, 16, 29, 64, 100])), len(toks) - lo)
            want_at = [k for k in range(c) if rng.random() < 0.5 or lo + k == len(toks) - 1]
            entries.append({"id": name, "tokens": toks[lo:lo + c], "want": want_at})
            expect.append(want[[lo + k for k in want_at]])
            limit.append(lim[[lo + k for k in want_at]])
            live[name][1] = lo + c
            if lo + c == len(toks):
                end.append(name)
        got = trace.step(entries, end)
        if got is not None:
            results.append((got.numpy(), np.concatenate(expect), np.concatenate(limit)))
        for name in end:
            del live[name]
            done += 1
    check(*(np.concatenate(x) for x in zip(*results)))
    sched = trace.engine.scheduler
    assert sched.block_manager.num_free_blocks == 10 and sched.slots.num_free == 4


SIZE = 70       # of the masks of the model below


def recall_model(folder, kind):
    """One layer; token 1 is the key of token 2: their score stands far above all others, wherever they stand, so that the value of a
    token far back decides the logits, and seeing or not seeing it shows."""
    width, dim = 96, 24
    entry = {"attention": dh.chunked(4, 2, dim, 16, SIZE, 1.0, 0.3, 4), "attention_2": dh.windowed(4, 2, dim, 16, SIZE, 2.0, 4, scaling=None),
             "parallel": dh.parallel(4, 2, dim, 16, SIZE, 1.0, right=0.01)}[kind]
    config = dh.make_config([entry], width=width, cap=100.0)
    w = dh.make_weights(config, seed=3)
    rng = np.random.default_rng(5)
    told, asked = np.linalg.qr(rng.standard_normal((width, 2)))[0].T * 40.0        # what marks token 1 and token 2
    maps = 2 if kind == "attention" else 1
    direction = np.zeros((2, maps, dim))
    direction[:, 0] = rng.standard_normal((2, dim)) * 0.8                          # the first map recalls
    direction[:, 0, :4] = 0.0                                                      # the rotated entries
    at = "l0.mix." + ("left." if kind == "parallel" else "")
    for name, mark, rows in ((at + "q", asked, np.repeat(direction, 2, 0)), (at + "k", told, direction)):
        away = np.eye(width) - np.outer(mark, mark) / (mark @ mark)
        w[name] = 0.3 * w[name] @ away + 0.25 * np.outer(rows.ravel(), mark) / np.sqrt(mark @ mark)
    if kind == "attention_2":
        for name in ("q", "k"):
            w[at + name + ".b"] *= 0.1
    w[at + "o"] = w[at + "o"] * 6.0
    w["l0.ls1"] = np.full(width, 2.0)
    w["bigram"] = w["bigram"] * 0.3
    w["embed"][1] += told
    w["embed"][2] += asked
    return Model(folder, "recall", config, {k: mh.bf16(v) for k, v in w.items()})


@DT
@pytest.mark.parametrize("kind", ["attention", "attention_2", "parallel"])
@pytest.mark.parametrize("at", [0, 1, 63, 69, 70, 127, 139, 140, 200])
def test_a_far_key_just_inside_and_just_outside_what_is_seen(gpu, tmp_path_factory, dtype, kind, at):
    m = recall_model(tmp_path_factory.mktemp("recall"), kind)
    n = 290
    rng = np.random.default_rng(at)
    toks = [int(t) for t in rng.integers(3, m.config["vocab"], n)]
    toks[at] = 1
    edge = at + SIZE if kind == "attention_2" else (at // SIZE + 1) * SIZE           # the first position that does not see it
    asks = sorted({p for p in (at + 1, at + 2, edge - 2, edge - 1, edge, edge + 1, edge + 30) if at < p < n})
    for p in asks:
        toks[p] = 2
    want, limit = m.limits(toks, dtype)
    without = ref.forward(m.config, m.weights, toks[:at] + [3] + toks[at + 1:])[0]
    shows = mh.row_errors(without, want)
    assert all((shows[p] > 0.2) if p < edge else (shows[p] < 0.1) for p in asks if p > at + 1), (asks, edge, shows[asks])
    trace = TraceReplay(m.folder, dtype, 320)
    for i, cuts in enumerate(([n], [at + 1] + [1] * (n - at - 1), [at + 1, n - at - 1], [37] * 7 + [31], [65] * 4 + [28, 2])):
        got = feed(trace, f"r{i}", toks, cuts)
        assert (mh.row_errors(got, want)[asks] <= limit[asks]).all()


@DT
def test_the_previous_token_across_cuts(gpu, models, dtype):
    """Only the second embedding tells these tokens apart: all rows of the first are equal."""
    config = dh.make_config([dh.windowed(size=1)], vocab=90)
    w = dh.make_weights(config, 2)
    w["embed"][:] = w["embed"][0]
    import tempfile
    with tempfile.TemporaryDirectory() as folder:
        m = Model(folder, "pairs", config, w)
        toks = mh.tokens(70, config, 3)
        want, limit = m.limits(toks, dtype)
        trace = TraceReplay(m.folder, dtype, 192)
        for i, cuts in enumerate(([70], [1] * 70, [2] * 35, [3, 1, 64, 2], [64, 1, 5])):
            check(feed(trace, f"r{i}", toks, cuts), want, limit)


@DT
def test_first_tokens_of_a_sequence_in_a_used_slot(gpu, models, dtype):
    """A new request starts from zero in the slot and the pages of one that left large values there."""
    m = models("wide")
    trace = TraceReplay(m.folder, dtype, 64 * 4)
    for r in range(6):
        toks = mh.tokens(40, m.config, 50 + r)
        want, limit = m.limits(toks, dtype)
        for t in tensors(trace.engine.model_runner.kv_cache):
            t.fill_(float("nan"))
        cuts = [[1] * 40, [2, 38], [40]][r % 3]
        check(feed(trace, f"r{r}", toks, cuts), want, limit)


def test_long_decoding_crosses_many_pages(gpu, models):
    m = models("mixed-layers")
    toks = mh.tokens(400, m.config, 7)
    trace = TraceReplay(m.folder, "float32", 448)
    check(feed(trace, "a", toks, [5] + [1] * 395), m.logits(toks), np.full(400, F32))


def test_long_prompt_in_bfloat16_and_its_parts(gpu, models):
    """Dense tiles behind a cached prefix, row by row, and segments of the recurrence give the same as one prompt."""
    m = models("wide")
    toks = mh.tokens(700, m.config, 8)
    want, limit = m.limits(toks, "bfloat16")
    trace = TraceReplay(m.folder, "bfloat16", 704)
    for i, cuts in enumerate(([700], [300, 400], [640, 60], [63] * 11 + [7])):
        check(feed(trace, f"r{i}", toks, cuts), want, limit)


@pytest.mark.parametrize("kw", [dict(), dict(enforce_eager=True), dict(max_model_len=64, max_num_batched_tokens=64),
                                dict(num_kvcache_blocks=6), dict(max_num_seqs=2)],
                         ids=["graphs", "eager", "small-budget", "preemption", "two-slots"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_scheduler(gpu, models, dtype, kw):
    m = models("mixed-layers" if dtype == "float32" else "state-space")
    eng = engine(m, dtype=dtype, **kw)
    prompts = [mh.tokens(n, m.config, 20 + n) for n in (1, 5, 40, 33, 17, 2)]
    outs = eng.generate(prompts, SamplingParams(0.0, 12, True))
    for p, o in zip(prompts, outs):
        assert len(o["token_ids"]) == 12
        greedy_is_right(m, p, o["token_ids"], 1e-3 if dtype == "float32" else 0.5)
    assert eng.scheduler.block_manager.num_free_blocks == eng.config.num_kvcache_blocks
    assert eng.scheduler.slots.num_free == eng.config.max_num_seqs


def test_pool_is_sized_from_free_memory_and_sampling_runs(gpu, models):
    m = models("mixed-layers")
    eng = engine(m, num_kvcache_blocks=-1, gpu_memory_utilization=0.05, enforce_eager=True)
    assert eng.config.num_kvcache_blocks > 1000
    outs = eng.generate([mh.tokens(9, m.config, 1)] * 3, SamplingParams(0.8, 5, True))
    assert all(len(o["token_ids"]) == 5 and max(o["token_ids"]) < m.config["vocab"] for o in outs)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_graph_replays_equal_eager_steps(gpu, models, dtype):
    """The state advances with every step, so the eager step runs on a saved copy of it first."""
    m = models("mixed-layers")
    eng = engine(m, dtype=dtype)
    runner, sched = eng.model_runner, eng.scheduler
    for n in (30, 31, 64):
        eng.add_request(mh.tokens(n, m.config, n), SamplingParams(0.0, 20, True))
    eng.step()
    for _ in range(5):
        portions = sched.schedule()
        assert [p.count for p in portions] == [1, 1, 1]
        run_bs = runner.prepare_decode([p.seq for p in portions])
        assert run_bs == 4
        kept = [(t, t.clone()) for t in tensors(runner.kv_cache)]
        with torch.inference_mode():
            eager = runner._decode_forward(run_bs).clone()
            for t, k in kept:
                t.copy_(k)
            torch.cuda.synchronize()
            replay = runner.decode_hidden(run_bs)[:3].clone()
            assert torch.equal(eager[:3], replay)
            tokens = runner.model.compute_logits(replay).argmax(-1).tolist()
        sched.postprocess(portions, tokens)


def test_command_lines(gpu, models, tmp_path):
    m = models("odd")
    run = subprocess.run([sys.executable, "-m", "infer_amd", "--model", m.folder, "--prompt-ids", "3,1,4", "--max-tokens", "4",
                          "--dtype", "float32", "--block-size", "32", "--num-blocks", "8", "--max-model-len", "64",
                          "--max-batched-tokens", "64", "--max-num-seqs", "2"], capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr
    greedy_is_right(m, [3, 1, 4], json.loads(run.stdout.splitlines()[-1])["token_ids"], 1e-3)
    toks = mh.tokens(7, m.config, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:4], "want": [1, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[4:], "want": [2]}], "end": ["x"]}]
    run = subprocess.run(["bin/trace_run", "--model", m.folder, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"],
                         input="\n".join(map(json.dumps, steps)), capture_output=True, text=True, timeout=100)
    assert run.returncode == 0 and [x for x in run.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1"], run.stderr
    want = m.logits(toks)
    check(np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, -1), want[[1, 3]], np.full(2, F32))
    check(np.fromfile(tmp_path / "1.f32", "<f4").reshape(1, -1), want[[6]], np.full(1, F32))
