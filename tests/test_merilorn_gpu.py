"""Merilorn through the engine (loader, cache and state pools, scheduler, captured decode graphs) against
``oracle/merilorn_ref.py``: whole prompts, portions, decoding, unequal batches, blocks and slots used again,
greedy generation.  float32 has to agree to rounding; in bfloat16 every position has a limit of its own, a
multiple of what rounding the activations alone does to it (a position whose mixer output nearly cancels is
sensitive, and stays so however the tokens are cut)."""
import subprocess
import sys

import numpy as np
import pytest
import torch

from infer_amd.llm_engine import LLMEngine
from infer_amd.sampling_params import SamplingParams
from infer_amd.trace import TraceReplay
from oracle import merilorn_ref as ref
from tests import merilorn_helpers as mh

pytestmark = pytest.mark.gpu
F32, BF16 = 2e-4, 5e-2

CONFIGS = {
    "mixed-layers": mh.small_config,
    # sizes that are multiples of nothing, one head, no grouping
    "odd": lambda: mh.make_config([mh.delta(heads=1, kv_heads=1, dim=10, vdim=6, conv=2), mh.latent(1, 12, 6, 10, 20, 0.3, ff=30)],
                                  width=50, vocab=77, embed_scale=1.0),
    # a window of the sizes of published models, few heads; partly rotated
    "wide": lambda: mh.make_config([mh.latent(2, 64, 32, 64, 256, 0.1, ff=128, dims=16), mh.delta(2, 1, 64, 64, 4)], width=128, vocab=100),
    # attention alone, recurrence alone
    "attention-only": lambda: mh.make_config([mh.latent(), mh.latent(scaling=None), mh.shared(mh.latent(), 0)]),
    "recurrence-only": lambda: mh.make_config([mh.delta(conv=1), mh.delta(heads=6, kv_heads=3, dim=8, vdim=8, conv=5, ff=40)]),
}


class Model:
    def __init__(self, folder, name):
        self.config = CONFIGS[name]()
        self.weights = mh.make_weights(self.config, seed=sum(map(ord, name)))
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


def feed(trace, name, toks, cuts, last=True):
    """One request alone in portions of the given sizes; logits of every token."""
    out, lo = [], 0
    for i, c in enumerate(cuts):
        end = [name] if last and i == len(cuts) - 1 else []
        out.append(trace.step([{"id": name, "tokens": toks[lo:lo + c], "want": list(range(c))}], end).numpy())
        lo += c
    assert lo == len(toks)
    return np.concatenate(out)


def check(got, want, limit):
    e = mh.row_errors(got, want)
    assert np.isfinite(got).all()
    bad = np.flatnonzero(e > limit)
    assert bad.size == 0, (bad[:10].tolist(), e[bad[:10]].tolist(), float(e.mean()))


DT = pytest.mark.parametrize("dtype", ["float32", "bfloat16"])


@DT
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_decode_and_portions(gpu, models, name, dtype):
    m = models(name)
    n = 150
    toks = mh.tokens(n, m.config, 1)
    want, limit = m.limits(toks, dtype)
    trace = TraceReplay(m.folder, dtype, 192)
    cuts = [[n], [n - 20] + [1] * 20, [2] * 20 + [64, 33, 1, 1, 3, 8], [1] * n, [66, 65, 2, 17], [1, 70, 1, 63, 15]]
    for i, c in enumerate(cuts):
        check(feed(trace, f"r{i}", toks, c), want, limit)
    sched = trace.engine.scheduler
    assert sched.block_manager.num_free_blocks == 3 and sched.slots.num_free == 4


@DT
def test_unequal_requests_in_one_batch_and_pages_and_slots_used_again(gpu, models, dtype):
    m = models("mixed-layers")
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
            check(got.numpy(), np.concatenate(expect), np.concatenate(limit))
        for name in end:
            del live[name]
            done += 1
    sched = trace.engine.scheduler
    assert sched.block_manager.num_free_blocks == 10 and sched.slots.num_free == 4


@DT
def test_steps_nobody_waits_for(gpu, models, dtype):
    """Decoded tokens whose logits nobody asks for are queued one behind the other."""
    m = models("mixed-layers")
    toks = mh.tokens(60, m.config, 6)
    trace = TraceReplay(m.folder, dtype, 64)
    for i, t in enumerate(toks):
        got = trace.step([{"id": "a", "tokens": [t], "want": [0] if i == 59 else []}], [])
    want, limit = m.limits(toks, dtype)
    check(got.numpy(), want[-1:], limit[-1:])


def test_long_decoding_crosses_many_pages(gpu, models):
    m = models("mixed-layers")
    toks = mh.tokens(400, m.config, 7)
    trace = TraceReplay(m.folder, "float32", 448)
    check(feed(trace, "a", toks, [5] + [1] * 395), m.logits(toks), F32)


def test_long_prompt_in_bfloat16_and_its_halves(gpu, models):
    """Expanded keys behind a cached prefix, and row by row, give the same as one prompt."""
    m = models("wide")
    toks = mh.tokens(700, m.config, 8)
    want, limit = m.limits(toks, "bfloat16")
    trace = TraceReplay(m.folder, "bfloat16", 704)
    for i, cuts in enumerate(([700], [300, 400], [640, 60], [63] * 11 + [7])):
        check(feed(trace, f"r{i}", toks, cuts), want, limit)


def engine(m, **kw):
    base = dict(kvcache_block_size=32, num_kvcache_blocks=40, max_num_seqs=8, max_model_len=256, max_num_batched_tokens=256)
    return LLMEngine(m.folder, **{**base, **kw})


def greedy_is_right(m, prompt, out, margin):
    """Every generated token is the oracle's best, or within ``margin`` of it."""
    seq = list(prompt) + out
    logits = m.logits(seq)[len(prompt) - 1:-1]
    gap = logits.max(-1) - logits[np.arange(len(out)), out]
    assert gap.max() <= margin, gap.max()


@pytest.mark.parametrize("kw", [dict(), dict(enforce_eager=True), dict(max_model_len=64, max_num_batched_tokens=64),
                                dict(num_kvcache_blocks=6), dict(max_num_seqs=2)],
                         ids=["graphs", "eager", "small-budget", "preemption", "two-slots"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_scheduler(gpu, models, dtype, kw):
    m = models("mixed-layers")
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
        keep = [{k: v.clone() for k, v in c.items()} if isinstance(c, dict) else c.clone() for c in runner.kv_cache]
        with torch.inference_mode():
            eager = runner._decode_forward(run_bs).clone()
            for c, k in zip(runner.kv_cache, keep):
                for a, b in ([(c[n], k[n]) for n in c] if isinstance(c, dict) else [(c, k)]):
                    a.copy_(b)
            torch.cuda.synchronize()
            replay = runner.decode_hidden(run_bs)[:3].clone()
            assert torch.equal(eager[:3], replay)
            tokens = runner.model.compute_logits(replay).argmax(-1).tolist()
        sched.postprocess(portions, tokens)


def test_command_lines(gpu, models, tmp_path):
    import json
    m = models("odd")
    run = subprocess.run([sys.executable, "-m", "infer_amd", "--model", m.folder, "--prompt-ids", "3,1,4", "--max-tokens", "4",
                          "--dtype", "float32", "--block-size", "32", "--num-blocks", "8", "--max-model-len", "64",
                          "--max-batched-tokens", "64", "--max-num-seqs", "2"], capture_output=True, text=True, timeout=100)
    assert run.returncode == 0, run.stderr
    greedy_is_right(m, [3, 1, 4], json.loads(run.stdout.splitlines()[-1])["token_ids"], 1e-3)
    toks = mh.tokens(7, m.config, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:4], "want": [1, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[4:6], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[6:], "want": [0]}], "end": ["x"]}]
    run = subprocess.run(["bin/trace_run", "--model", m.folder, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"],
                         input="\n".join(map(json.dumps, steps)), capture_output=True, text=True, timeout=100)
    assert run.returncode == 0 and [x for x in run.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"], run.stderr
    want = m.logits(toks)
    check(np.fromfile(tmp_path / "0.f32", "<f4").reshape(2, -1), want[[1, 3]], F32)
    check(np.fromfile(tmp_path / "2.f32", "<f4").reshape(1, -1), want[[6]], F32)
    assert not (tmp_path / "1.f32").exists()
