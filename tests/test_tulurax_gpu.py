"""Tulurax through the engine (loader, cache and state pools, scheduler, captured decode graphs) against
``oracle/tulurax_ref.py``: whole prompts, portions, decoding, unequal batches, blocks and slots used again, greedy
generation.  float32 has to agree to rounding; in bfloat16 every position has a limit of its own, a multiple of what
rounding the activations alone does to it."""
import json
import subprocess
import sys

import numpy as np
import pytest
import torch

from infer_amd.sampling_params import SamplingParams
from infer_amd.trace import TraceReplay
from oracle import tulurax_ref as ref
from tests import merilorn_helpers as mh, tulurax_helpers as th
from tests.test_dogetar_gpu import tensors
from tests.test_merilorn_gpu import BF16, DT, F32, check, engine, feed, greedy_is_right

pytestmark = pytest.mark.gpu

CONFIGS = {
    "mixed-layers": th.small_config,
    # sizes that are multiples of nothing, one head, one key of temperature per token, no cap
    "odd": lambda: th.make_config([th.layer(1, 1, 10, 7, 0.6, (0.4, 1), (0.9,), 9, 5, ff=30), th.layer(3, 3, 13, 5, 0.5, (2.0, 7), (0.99, 0.3), 6, 11, ff=None),
                                   th.layer(6, 3, 20, 12, 0.4, None, (1.0,), 10, 6, ff=17)], width=50, vocab=77, cap=None),
    # heads of the sizes of published models: everything on the matrix pipe
    "wide": lambda: th.make_config([th.layer(8, 2, 64, 64, 0.125, (0.5, 64), (0.9, 0.99, 0.999, 1 - 2.0 ** -10), 64, 64, ff=128),
                                    th.layer(12, 12, 64, 128, 0.1, (0.3, 100), (0.95, 0.9995), 128, 128, 1.2, 0.3, 96),
                                    th.layer(20, 4, 128, 64, 0.09, None, (0.9,), 32, 64, ff=64)], width=128, vocab=100, eps=1e-6),
    # scales and constants that drop out
    "ones": lambda: th.make_config([th.layer(4, 4, 16, 16, 0.25, (0.0, 5), (0.9,), 16, 16, 1.0, 1.0), th.layer(2, 1, 32, 8, 0.2, None, (0.7, 0.7), 8, 32, 1.0, 1.0)],
                                   eps=1e-2, embed_scale=1.0, logit_scale=1.0),
}


class Model:
    def __init__(self, folder, name, config=None, weights=None):
        self.config = config or CONFIGS[name]()
        self.weights = weights or th.make_weights(self.config, seed=sum(map(ord, name)))
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
@pytest.mark.parametrize("name", ["mixed-layers", "wide"])
def test_unequal_requests_in_one_batch_and_pages_and_slots_used_again(gpu, models, name, dtype):
    m = models(name)
    trace = TraceReplay(m.folder, dtype, 640)
    rng = np.random.default_rng(4)
    live, done, made = {}, 0, 0
    while done < 10:
        while len(live) < 4 and made < 10:
            n = [130, 3, 70, 1, 129, 64, 90, 2, 65, 100][made]
            toks = mh.tokens(n, m.config, 100 + made)
            live[f"q{made}"] = [toks, 0, *m.limits(toks, dtype)]
            made += 1
        entries, end, expect, limit = [], [], [], []
        for request in sorted(live, key=lambda _: rng.random()):
            toks, lo, want, lim = live[request]
            if rng.random() < 0.2:
                continue                               # left out of this step
            c = min(int(rng.choice([1, 1, 2, 3, 16, 29, 64, 100])), len(toks) - lo)
            want_at = [k for k in range(c) if rng.random() < 0.5 or lo + k == len(toks) - 1]
            entries.append({"id": request, "tokens": toks[lo:lo + c], "want": want_at})
            expect.append(want[[lo + k for k in want_at]])
            limit.append(lim[[lo + k for k in want_at]])
            live[request][1] = lo + c
            if lo + c == len(toks):
                end.append(request)
        got = trace.step(entries, end)
        if got is not None:
            check(got.numpy(), np.concatenate(expect), np.concatenate(limit))
        for request in end:
            del live[request]
            done += 1
    sched = trace.engine.scheduler
    assert sched.block_manager.num_free_blocks == 10 and sched.slots.num_free == 4


def recall_model(folder):
    """One layer; token 1 is the key of token 2 for one head, whose weights two other heads apply to their own values: their score
    stands far above all others, wherever they stand, so that seeing, losing or misplacing token 1 shows."""
    width, heads, dim = 96, 4, 24
    config = th.make_config([th.layer(heads, 2, dim, 16, 0.5, (0.5, 64), (0.5,), right=0.01, ff=None)], width=width, cap=200.0)
    w = th.make_weights(config, seed=3)
    rng = np.random.default_rng(5)
    told, asked = np.linalg.qr(rng.standard_normal((width, 2)))[0].T * 20.0         # what marks token 1 and token 2
    direction = rng.standard_normal((2, dim)) * 0.8
    for name, mark, rows in (("q", asked, np.repeat(direction, 2, 0)), ("k", told, direction)):
        away = np.eye(width) - np.outer(mark, mark) / (mark @ mark)
        w["l0.mix.left." + name] = 0.1 * w["l0.mix.left." + name] @ away + np.outer(rows.ravel(), mark) / np.sqrt(mark @ mark)
    w["l0.mix.left.talk"] = np.array([[0.0, 1.0, 0.0, 0.0], [0.0, 0.0, 0.0, 0.0], [0.0, -1.0, 0.0, 0.0], [0.0, 0.0, 0.0, 0.0]])
    w["l0.mix.left.o"] = w["l0.mix.left.o"] * 3.0
    for norm in ("embed.norm", "l0.norm1", "final.norm"):                           # close to linear
        w[norm + ".alpha"], w[norm] = np.asarray(0.25), np.ones(width)
        w[norm + ".b"] *= 0.1
    scale = config["embedding"]["scale"]
    w["embed"] = 0.3 * w["embed"]
    w["embed"][1] += told / scale
    w["embed"][2] += asked / scale
    return Model(folder, "recall", config, {k: mh.bf16(v) for k, v in w.items()})


@DT
@pytest.mark.parametrize("at", [0, 1, 31, 32, 63, 64, 127, 200])
def test_a_far_key_at_page_borders(gpu, tmp_path_factory, dtype, at):
    m = recall_model(tmp_path_factory.mktemp("recall"))
    n = 290
    rng = np.random.default_rng(at)
    toks = [int(t) for t in rng.integers(3, m.config["vocab"], n)]
    toks[at] = 1
    asks = sorted({p for p in (at + 1, at + 2, at + 31, at + 32, at + 64, 255, 256, 257, 289) if at < p < n})
    for p in asks:
        toks[p] = 2
    want, limit = m.limits(toks, dtype)
    without = m.logits(toks[:at] + [3] + toks[at + 1:])
    assert (mh.row_errors(without, want)[asks] > 0.3).all(), mh.row_errors(without, want)[asks]
    trace = TraceReplay(m.folder, dtype, 320)
    for i, cuts in enumerate(([n], [at + 1] + [1] * (n - at - 1), [at + 1, n - at - 1], [37] * 7 + [31], [65] * 4 + [28, 2])):
        got = feed(trace, f"r{i}", toks, cuts)
        assert (mh.row_errors(got, want)[asks] <= limit[asks]).all()


@DT
def test_the_temperature_steps_where_it_should(gpu, tmp_path_factory, dtype):
    """The same token everywhere but for one key: what changes along the sequence is the temperature, and the sink's share."""
    config = th.make_config([th.layer(2, 2, 16, 16, 0.4, (3.0, 40), (0.5,), right=0.01, ff=None)], cap=100.0)
    w = th.make_weights(config, 9)
    m = Model(tmp_path_factory.mktemp("steps"), "steps", config, w)
    toks = [7] + [5] * 129
    want, limit = m.limits(toks, dtype)
    trace = TraceReplay(m.folder, dtype, 192)
    shift = np.abs(np.diff(want, axis=0)).max(-1)
    assert all(shift[p - 1] > 3 * shift[p] for p in (39, 79, 119))               # position 39 is the first of the second step
    for i, cuts in enumerate(([130], [1] * 130, [39, 1, 40, 50], [64, 66])):
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
        check(feed(trace, f"r{r}", toks, [[1] * 40, [2, 38], [40]][r % 3]), want, limit)


def test_long_decoding_crosses_many_pages(gpu, models):
    m = models("mixed-layers")
    toks = mh.tokens(400, m.config, 7)
    trace = TraceReplay(m.folder, "float32", 448)
    check(feed(trace, "a", toks, [5] + [1] * 395), m.logits(toks), np.full(400, F32))


def test_long_prompt_in_bfloat16_and_its_parts(gpu, models):
    """Tiles behind a cached prefix, row by row, and segments of the recurrence give the same as one prompt."""
    m = models("wide")
    toks = mh.tokens(700, m.config, 8)
    want, limit = m.limits(toks, "bfloat16")
    trace = TraceReplay(m.folder, "bfloat16", 704)
    for i, cuts in enumerate(([700], [300, 400], [640, 60], [63] * 11 + [7])):
        check(feed(trace, f"r{i}", toks, cuts), want, limit)


@pytest.mark.parametrize("kw", [dict(), dict(enforce_eager=True), dict(max_model_len=64, max_num_batched_tokens=64),
                                dict(num_kvcache_blocks=6), dict(max_num_seqs=2)],
                         ids=["graphs", "eager", "small-budget", "preemption", "two-slots"])
@DT
def test_greedy_generation_through_the_scheduler(gpu, models, dtype, kw):
    m = models("mixed-layers" if dtype == "float32" else "wide")
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


@pytest.mark.parametrize("name", ["mixed-layers", "wide"])
@DT
def test_graph_replays_equal_eager_steps(gpu, models, name, dtype):
    """The state advances with every step, so the eager step runs on a saved copy of it first."""
    m = models(name)
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
