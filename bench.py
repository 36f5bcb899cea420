"""Benchmark of the paged KV-cache hot path on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W]

A step is one paged decode attention (streaming kernel + merge kernel) over the Qwen3-8B-shaped
decode batch (32 query heads, 8 KV heads, head_dim 128, block 256, batch 64, context lengths
uniform in [512, 4096], block tables shuffled over a pool 1.2x the need).  Inputs are resident
in HBM before the clock starts; the GPU is brought to its steady clocks by a quarter of a second of
the same op (untimed) before the W warm-up steps and the K timed steps.  Successive steps walk over several independent copies of the
cache (as successive layers of a model do) so that the 256 MB Infinity Cache cannot serve the
reads.  Prints one JSON line.

Besides the headline the line carries: the roofline of the dominant kernel, the decode op over the
range of shapes the target names (``decode_curve``), the KV append at prefill size, the fused
front end, the prefill attention, the CPU baselines, and the end-to-end run of the engine.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

import torch

HBM_PEAK_GBS = 8000.0
ROOT = os.path.dirname(os.path.abspath(__file__))

# HBM bytes per launch of the decode streaming kernel on the headline workload.  This is a RECORDED
# figure, not measured by this run: two `rocprofv3 --pmc` passes of `python3 bench.py --counters`
# (FETCH_SIZE, then WRITE_SIZE, KiB per dispatch, each scaled by what the same counter reads for the
# 1 GiB plain copy that run launches first) gave 630,159 KiB read + 2,992 KiB written; the summary is
# profiles/decode_cfg2_hbm_counters.txt.  The workload is seeded, so the figure only moves when the
# kernel's access pattern does; it has to be re-recorded then.
MEASURED_TRAFFIC_BYTES = (630159 + 2992) * 1024
TRAFFIC_SOURCE = "recorded: profiles/decode_cfg2_hbm_counters.txt (rocprofv3 --pmc FETCH_SIZE / WRITE_SIZE)"


def gpu_time_ms(fn, iters, warmup):
    """Average milliseconds per call of ``fn`` over ``iters`` calls, HIP events on the current stream."""
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    start = torch.cuda.Event(enable_timing=True)
    stop = torch.cuda.Event(enable_timing=True)
    start.record()
    for _ in range(iters):
        fn()
    stop.record()
    torch.cuda.synchronize()
    return start.elapsed_time(stop) / iters


def gpu_time_ms_median(fn, iters, warmup, runs=5):
    """Median over ``runs`` of gpu_time_ms(fn, iters, ...): for the secondary figures, whose launches are short
    enough for one slow host moment (or the clock ramp of the first run) to shift a single average."""
    times = sorted(gpu_time_ms(fn, iters, warmup if r == 0 else 2) for r in range(runs))
    return times[len(times) // 2]


# ------------------------------------------------------------------------------------------ CPU legs
def _host_threads():
    cores = os.cpu_count() or 1
    cores = min(cores, int(os.environ.get("OMP_NUM_THREADS", cores)))
    torch.set_num_threads(cores)
    return cores


def _median_time(fn, min_seconds, min_runs=3, max_runs=50):
    fn()
    times = []
    t_end = time.perf_counter() + min_seconds
    while len(times) < min_runs or (time.perf_counter() < t_end and len(times) < max_runs):
        t0 = time.perf_counter()
        fn()
        times.append(time.perf_counter() - t0)
    times.sort()
    return times[len(times) // 2], len(times)


def _cpu_model():
    """The host CPU's model string (first `model name` of /proc/cpuinfo), for the baseline's record."""
    try:
        with open("/proc/cpuinfo") as f:
            for ln in f:
                if ln.lower().startswith("model name"):
                    return ln.split(":", 1)[1].strip()
    except OSError:
        pass
    return "unknown"


def cpu_baseline(sample_seqs=16, min_seconds=8.0):
    """The CPU restatement of the same path (gather + SDPA, oracle/torch_path.py) on the host cores,
    over a bounded sample of the same workload: the first ``sample_seqs`` sequences of the batch."""
    from infer_amd import workloads
    from oracle import torch_path
    cores = _host_threads()
    lengths = workloads.cfg2_lengths()[:sample_seqs]
    wl = workloads.make_decode_workload("cfg2-sample", lengths, 32, 8, seed=0, q_scale=128 ** -0.5)
    med, runs = _median_time(lambda: torch_path.paged_decode_torch(wl.q, wl.k_cache, wl.v_cache, wl.block_table,
                                                                   wl.context_lens, wl.scale), min_seconds)
    return {
        "value": round(wl.decode_bytes / med / 1e9, 3), "unit": "GB/s", "cores": cores, "kind": "port",
        "sample": f"first {sample_seqs} of the 64 sequences ({sum(lengths)} tokens, "
                  f"{wl.decode_bytes / 1e6:.1f} MB algorithmic), median of {runs} runs, "
                  f"torch {torch.get_num_threads()} threads",
        "cpu_model": _cpu_model(),
    }


def cpu_baselines_other(p3_cpu):
    """The same CPU port on the other named configurations, each on a bounded sample: the whole
    Qwen3-0.6B-shaped step (cfg1), one of the eight 32,768-token sequences of the long-context step
    (cfg4), and the prefill-sized KV append (cfg3, ``index_copy_`` as the reference's torch path)."""
    from infer_amd import workloads
    from oracle import torch_path
    cores = _host_threads()
    out = {}
    w1 = workloads.cfg1()
    med, runs = _median_time(lambda: torch_path.paged_decode_torch(w1.q, w1.k_cache, w1.v_cache, w1.block_table,
                                                                   w1.context_lens, w1.scale), 2.0)
    out["cfg1_decode"] = {"value": round(w1.decode_bytes / med / 1e9, 3), "unit": "GB/s", "cores": cores, "kind": "port",
                          "sample": f"whole step (4 sequences, {w1.decode_bytes / 1e6:.2f} MB), median of {runs} runs"}
    w4 = workloads.make_decode_workload("cfg4-sample", [32768], 64, 8, nblk=160, seed=0)
    med, runs = _median_time(lambda: torch_path.paged_decode_torch(w4.q, w4.k_cache, w4.v_cache, w4.block_table,
                                                                   w4.context_lens, w4.scale), 4.0)
    out["cfg4_decode"] = {"value": round(w4.decode_bytes / med / 1e9, 3), "unit": "GB/s", "cores": cores, "kind": "port",
                          "sample": f"one of the 8 sequences of 32,768 tokens ({w4.decode_bytes / 1e6:.1f} MB), "
                                    f"median of {runs} runs"}
    kc, vc = p3_cpu.k_cache.clone(), p3_cpu.v_cache.clone()
    med, runs = _median_time(lambda: torch_path.append_torch(p3_cpu.k_new, p3_cpu.v_new, kc, vc, p3_cpu.slot_mapping), 3.0)
    out["cfg3_append"] = {"value": round(p3_cpu.append_bytes / med / 1e9, 3), "unit": "GB/s", "cores": cores,
                          "kind": "port", "sample": f"whole step ({int(p3_cpu.slot_mapping.numel())} rows, "
                                                    f"{p3_cpu.append_bytes / 1e6:.1f} MB), median of {runs} runs"}
    w2 = workloads.make_decode_workload("cfg2-append", workloads.cfg2_lengths(), 32, 8, nblk=800, seed=0)
    kc2, vc2 = w2.k_cache, w2.v_cache
    med, runs = _median_time(lambda: torch_path.append_torch(w2.k_new, w2.v_new, kc2, vc2, w2.slot_mapping), 1.0)
    out["cfg2_append_64_rows"] = {"value": round(med * 1e6, 2), "unit": "us", "cores": cores, "kind": "port",
                                  "sample": f"whole step (64 rows), median of {runs} runs"}
    return out


# ------------------------------------------------------------------------------------------ end to end
def run_e2e(args):
    """End-to-end decode through the engine: random-init model of a published Qwen3 shape, batch of
    random-token prompts with lengths uniform in [128, 1024], greedy decoding, KV pool filling the
    free HBM, decode step replayed as a HIP graph.  The first ``--e2e-check`` decode steps run twice on
    the same state, eagerly and as the graph replay, and must sample the same tokens from finite
    logits; at the end every cache block must be back in the pool.  Prints one JSON line."""
    import numpy as np
    from infer_amd import config as C
    from infer_amd.llm_engine import LLMEngine
    from infer_amd.sampling_params import SamplingParams
    hf = {"8b": C.qwen3_8b, "0.6b": C.qwen3_0_6b, "32b": C.qwen3_32b}[args.e2e_model]()
    t0 = time.perf_counter()
    engine = LLMEngine(hf_config=hf, max_num_seqs=max(args.e2e_batch, 16), max_model_len=4096,
                       max_num_batched_tokens=16384, enforce_eager=args.e2e_eager, seed=0)
    torch.cuda.synchronize()
    t_init = time.perf_counter() - t0
    rng = np.random.default_rng(0)
    lengths = rng.integers(128, 1025, size=args.e2e_batch)
    prompts = [[int(t) for t in rng.integers(0, hf.vocab_size, size=int(n))] for n in lengths]
    sp = SamplingParams(temperature=0.0, max_tokens=args.e2e_new, ignore_eos=True)
    runner = engine.model_runner
    check = {"steps": 0, "tokens_equal": True, "logits_finite": True, "max_logit_diff": 0.0}
    if not args.e2e_eager and args.e2e_check > 0:
        # A decode step is idempotent on the cache (the same row goes to the same slot), so the first
        # steps run twice on the same state, eagerly and then as the graph replay: same greedy tokens,
        # finite logits.  The time the check adds is kept apart and taken out of the clock below.
        replay = runner.decode_hidden
        left = [args.e2e_check]

        def checked_decode_hidden(run_bs):
            if left[0] <= 0 or run_bs not in runner.graphs:
                return replay(run_bs)
            left[0] -= 1
            n = int((runner.h_seq_lens[:run_bs] > 0).sum())
            t0 = time.perf_counter()
            eager = runner.model.compute_logits(runner._decode_forward(run_bs)[:n]).float()
            torch.cuda.synchronize()
            check["seconds"] = check.get("seconds", 0.0) + time.perf_counter() - t0
            hidden = replay(run_bs)
            torch.cuda.synchronize()             # the replay itself is the step's own time, not the check's
            t0 = time.perf_counter()
            graph = runner.model.compute_logits(hidden[:n]).float()
            check["steps"] += 1
            check["tokens_equal"] &= bool(torch.equal(eager.argmax(-1), graph.argmax(-1)))
            check["logits_finite"] &= bool(torch.isfinite(eager).all() and torch.isfinite(graph).all())
            check["max_logit_diff"] = max(check["max_logit_diff"], float((eager - graph).abs().max()))
            torch.cuda.synchronize()
            check["seconds"] += time.perf_counter() - t0
            return hidden
        runner.decode_hidden = checked_decode_hidden
    t0 = time.perf_counter()
    outs = engine.generate(prompts, sp)
    torch.cuda.synchronize()
    wall = time.perf_counter() - t0
    st = engine.stats
    assert all(len(o["token_ids"]) == args.e2e_new for o in outs)
    pool = engine.scheduler.block_manager
    pool_ok = pool.num_free_blocks == engine.config.num_kvcache_blocks and len(pool.used_block_ids) == 0
    # the checked steps stay in the count; what the check added to them (the eager run, the comparison)
    # is taken out of the clock
    timed_steps = st["decode_steps"]
    timed_s = st["decode_s"] - check.get("seconds", 0.0)
    dec_tps = st["decode_tokens"] / timed_s if timed_s else 0.0
    print(json.dumps({
        "metric": "end-to-end greedy decode throughput through the engine", "value": round(dec_tps, 1),
        "unit": "tokens/s", "n_gpus": 1, "higher_is_better": True, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": f"cfg5: random-init Qwen3-{args.e2e_model} decode, batch {args.e2e_batch}, prompts "
                               f"U[128,1024], {args.e2e_new} greedy tokens, hipGraph={not args.e2e_eager}"},
        "decode_steps": st["decode_steps"], "decode_ms_per_step": round(1e3 * timed_s / max(timed_steps, 1), 3),
        "check_seconds_excluded": round(check.get("seconds", 0.0), 4),
        "prefill_tokens_per_s": round(st["prefill_tokens"] / st["prefill_s"], 1) if st["prefill_s"] else None,
        "prefill_steps": st["prefill_steps"], "generate_wall_s": round(wall, 2), "init_s": round(t_init, 1),
        "num_kvcache_blocks": engine.config.num_kvcache_blocks,
        "kv_pool_GB": round(runner.kv_cache.numel() * 2 / 1e9, 1),
        "graphs": len(runner.graphs),
        "checked_decode_steps": check["steps"], "tokens_equal": bool(check["tokens_equal"]) if check["steps"] else None,
        "logits_finite": bool(check["logits_finite"]) if check["steps"] else None,
        "max_logit_diff_eager_vs_graph": check["max_logit_diff"] if check["steps"] else None,
        "pool_all_blocks_free_at_end": bool(pool_ok)}))
    if check["steps"] and not (check["tokens_equal"] and check["logits_finite"]):
        sys.exit(3)
    if not pool_ok:
        sys.exit(4)


# ------------------------------------------------------------------------------------------ hybrid models
BF16_PEAK_TFLOPS, F32_MFMA_PEAK_TFLOPS = 2500.0, 157.3
# width, feed-forward, attention heads, layers: layers of the size of Qwen3-0.6B's and Qwen3-8B's
HYBRID_SIZES = {"0.6b": (1024, 3072, 16, 16), "8b": (4096, 12288, 32, 12)}


def hybrid_config(size):
    """Merilorn of a published model's width: three delta-rule layers to one of latent attention, all with a
    feed-forward; latent of 512 + 64, heads of 128."""
    from infer_amd.config import LayerSpec, MerilornConfig
    width, ff, heads, layers = HYBRID_SIZES[size]
    latent = {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "scale": 192 ** -0.5,
              "rot": {"base": 1e5, "dims": 64, "scaling": {"factor": 2.0, "original": 32768, "fast": 16.0, "slow": 2.0}}}
    delta = {"heads": heads, "kv_heads": heads, "dim": 128, "vdim": 128, "conv": 4, "decay_rank": 128, "gate_rank": 128}
    specs = [LayerSpec("latent_attention", latent, ff, i) if i % 4 == 3 else LayerSpec("channel_delta", delta, ff, i)
             for i in range(layers)]
    return MerilornConfig(vocab_size=151936, hidden_size=width, layers=specs, embedding_scale=width ** 0.5)


def vokelix_config(size):
    """Vokelix of a published model's width: two lightning layers, one of retention, one of grouped attention with 8 key
    heads, all with a feed-forward; every second attention layer uses the keys of the one before; heads of 128."""
    from infer_amd.config import LayerSpec, VokelixConfig
    width, ff, heads, layers = HYBRID_SIZES[size]
    attn = {"heads": heads, "kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
            "rot": {"base": 1e6, "dims": 64, "scaling": {"factor": 4.0, "original": 8192, "fast": 16.0, "slow": 2.0}}}
    decay = [1.0 - 2.0 ** (-4.0 - 7.0 * h / heads) for h in range(heads)]
    linear = {"heads": heads, "dim": 128, "vdim": 128, "decay": decay}
    kinds = {0: ("lightning", linear), 1: ("lightning", linear), 2: ("retention", {**linear, "rot": {"base": 1e4, "dims": 128}})}
    specs = []
    for i in range(layers):
        kind, mixer = kinds.get(i % 4, ("attention", {**attn, "kv_from": i - 4} if i % 8 == 7 else attn))
        specs.append(LayerSpec(kind, mixer, ff, i))
    return VokelixConfig(vocab_size=151936, hidden_size=width, layers=specs, residual_alpha=2.0)


def dogetar_config(size):
    """Dogetar of a published model's width: eight layers of which four run twice.  Every fourth has biased attention beside a state
    space and a dense feed-forward; the others attention of two maps in chunks or windowed attention, and a mixture whose chosen experts and
    shared expert together are as wide as the feed-forward."""
    from infer_amd.config import DogetarConfig, LayerLoop, LayerSpec
    width, ff, heads, runs = HYBRID_SIZES[size]
    rot = {"base": 5e5, "dims": 64}
    attn = {"kv_heads": 8, "dim": 128, "vdim": 128, "scale": 128 ** -0.5}
    two_maps = {**attn, "heads": heads, "dim": 64, "diff": 0.5, "scale": 0.125, "mask": {"size": 2048}, "rot": rot}
    window = {**attn, "heads": heads, "mask": {"size": 1024}, "rot": {**rot, "scaling": {"factor": 4.0, "original": 8192, "low": 1.0, "high": 4.0}}}
    parallel = {"left": {**attn, "heads": heads // 2, "mask": {"size": 2048}}, "left_scale": 1.0, "right_scale": 1.0,
                "right": {"heads": heads * 2, "vdim": 64, "state": 128, "groups": 2, "conv": 4, "norm_groups": 2}}
    dense = {"kind": "dense", "ff": ff, "limit": 7.0}
    moe = {"kind": "moe", "expert": {"ff": ff // 4}, "shared": {"ff": ff // 4},
           "router": {"experts": 14, "identity": 2, "top": 3, "scale": 2.0, "groups": {"count": 4, "keep": 2}}}
    kinds = [("parallel", parallel, dense), ("attention", two_maps, moe), ("attention_2", window, moe), ("attention", two_maps, moe)]
    layers = runs * 2 // 3
    specs = [LayerSpec(kind, mixer, ff if mlp is dense else None, i, mlp) for i in range(layers) for kind, mixer, mlp in (kinds[i % 4],)]
    return DogetarConfig(vocab_size=151936, hidden_size=width, layers=specs, bigram={"buckets": 65521, "mul_prev": 131, "mul_cur": 17},
                         loop=LayerLoop(2, 2 + runs - layers, 2), logit_softcap=30.0)


def tulurax_config(size):
    """Tulurax of a published model's width: half of the heads talking (8 key heads), half retention, all of 128; a feed-forward without a
    gate in every layer, so half again as wide to have as many weights as one with a gate."""
    from infer_amd.config import LayerSpec, TuluraxConfig
    width, ff, heads, layers = HYBRID_SIZES[size]
    half = heads // 2
    mixer = {"left": {"heads": half, "kv_heads": min(half, 8), "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "q_temp": {"coef": 0.1, "every": 8192}},
             "left_scale": 0.7, "right_scale": 0.7,
             "right": {"heads": half, "dim": 128, "vdim": 128, "decay": [1.0 - 2.0 ** (-4.0 - 7.0 * h / half) for h in range(half)]}}
    return TuluraxConfig(vocab_size=151936, hidden_size=width, layers=[LayerSpec("parallel", mixer, ff * 3 // 2, i) for i in range(layers)],
                         embedding_scale=1.0, logit_scale=1.0, logit_softcap=30.0)


def hybrid_engine_point(size, model, batch, prompt, new):
    """Prefill and decode throughput of the engine on ``batch`` prompts of ``prompt`` random tokens."""
    import numpy as np
    from infer_amd import config as C
    from infer_amd.llm_engine import LLMEngine
    from infer_amd.sampling_params import SamplingParams
    width, ff, heads, layers = HYBRID_SIZES[size]
    if model == "qwen3":
        hf = C.ModelConfig(hidden_size=width, intermediate_size=ff, num_hidden_layers=layers, num_attention_heads=heads, num_key_value_heads=8)
    else:
        hf = {"merilorn": hybrid_config, "vokelix": vokelix_config, "dogetar": dogetar_config,
              "tulurax": tulurax_config}[model](size)
    blocks = batch * (-(-(prompt + new) // 256) + 1)
    engine = LLMEngine(hf_config=hf, max_num_seqs=max(batch, 16), max_model_len=prompt + new + 1,
                       max_num_batched_tokens=16384, num_kvcache_blocks=blocks, seed=0)
    rng = np.random.default_rng(0)
    params = SamplingParams(temperature=0.0, max_tokens=new, ignore_eos=True)
    for i in range(2):                      # the first pass warms up
        for key in engine.stats:
            engine.stats[key] = 0
        prompts = [[int(t) for t in rng.integers(0, hf.vocab_size, size=prompt)] for _ in range(batch)]
        outs = engine.generate(prompts, params)
        assert all(len(o["token_ids"]) == new for o in outs)
    st = engine.stats
    point = {"model": model, "layers_like": size, "layers": layers, "batch": batch, "prompt": prompt, "new_tokens": new,
             "prefill_tokens_per_s": round(st["prefill_tokens"] / st["prefill_s"], 1),
             "decode_tokens_per_s": round(st["decode_tokens"] / st["decode_s"], 1),
             "decode_ms_per_step": round(1e3 * st["decode_s"] / st["decode_steps"], 3)}
    del engine
    torch.cuda.empty_cache()
    return point


def roofline_table(dev):
    """A dict of timed kernels, and the functions that time one against the memory bandwidth or a matrix peak."""
    out = {}

    def rnd(*shape, dtype=torch.bfloat16):
        return torch.randn(*shape, dtype=dtype, device=dev)

    def hbm(name, nbytes, fn, note=""):
        ms = gpu_time_ms_median(fn, 20, 5)
        out[name] = {"us": round(ms * 1e3, 2), "bound": "hbm", "GBps": round(nbytes / ms / 1e6, 1),
                     "frac": round(nbytes / ms / 1e6 / HBM_PEAK_GBS, 4), **({"note": note} if note else {})}

    def mfma(name, flops, peak, fn, note=""):
        ms = gpu_time_ms_median(fn, 20, 5)
        out[name] = {"us": round(ms * 1e3, 2), "bound": "mfma", "TFLOPs": round(flops / ms / 1e9, 1),
                     "frac": round(flops / ms / 1e9 / peak, 4), **({"note": note} if note else {})}

    return out, rnd, hbm, mfma


def hybrid_kernels(heads=32, width=4096, ff=12288):
    """Every kernel of the design at the sizes of an 8B model's layers, with what bounds it, beside the like kernel of
    Qwen3 at the same sizes."""
    from infer_amd import hybrid_ops as ho, ops, workloads
    from infer_amd.layers import yarn_rotary_table
    from infer_amd.step_plan import CHUNK
    dev, bf = torch.device("cuda:0"), torch.bfloat16
    out, rnd, hbm, mfma = roofline_table(dev)

    # ---- decode attention, batch 64 x ctx 4096
    b, ctx, bs, row, rank, dim, rot, vdim = 64, 4096, 256, 576, 512, 128, 64, 128
    nblk = b * ctx // bs
    cache = rnd(nblk, bs, row)
    tables = torch.randperm(nblk, device=dev).to(torch.int32).view(b, -1)
    lens = torch.full((b,), ctx, dtype=torch.int32, device=dev)
    for h in (16, heads, 128):
        qx = rnd(b, h, row)
        hbm(f"latent_attention decode, {h} heads", b * ctx * row * 2, lambda: ho.latent_attention(qx, cache, tables, lens, 0.07, rank))
    wl = workloads.make_decode_workload("b64-ctx4096", [ctx] * b, heads, 8, seed=0, q_scale=128 ** -0.5, device=dev, device_fill=True)
    o = torch.empty((b, heads, 128), dtype=bf, device=dev)
    hbm("qwen3: paged decode attention", wl.decode_bytes,
        lambda: ops.paged_attn_decode(wl.q, wl.k_cache, wl.v_cache, wl.block_table, wl.context_lens, wl.scale, o))
    del wl

    # ---- prefill attention, 8 prompts of 2048
    n, sq = 8, 2048
    cu = torch.arange(0, n + 1, dtype=torch.int32, device=dev) * sq
    rows = rnd(n * sq, row)
    q, kv, gate = rnd(n * sq, heads * (dim + rot)), rnd(n * sq, heads * (dim + vdim)), rnd(n * sq, heads)
    at = torch.empty((n * sq, heads * vdim), dtype=bf, device=dev)
    pairs = n * sq * (sq + 1) // 2
    mfma("latent_prefill, 8 x 2048", 2 * heads * (dim + rot + vdim) * pairs, BF16_PEAK_TFLOPS,
         lambda: ho.latent_prefill(q, kv[:, :heads * dim], rows[:, rank:], kv[:, heads * dim:], gate, at, cu, cu, sq, heads, dim, rot, vdim, 0.07))
    q3, k3 = rnd(n * sq, heads, 128), rnd(n * sq, 8, 128)
    mfma("qwen3: prefill attention, 8 x 2048", 4 * heads * 128 * pairs, BF16_PEAK_TFLOPS,
         lambda: ops.flash_attn_varlen_func(q3, k3, k3, max_seqlen_q=sq, cu_seqlens_q=cu, max_seqlen_k=sq, cu_seqlens_k=cu))
    seqs = torch.arange(n, dtype=torch.int32, device=dev)
    hbm("latent_gather, 16384 rows", 2 * n * sq * row * 2, lambda: ho.latent_gather(cache, tables[:n], seqs, cu, n * sq, sq))
    del q, kv, q3, k3

    # ---- front end and per-head products
    table = yarn_rotary_table(rot, 8192, 1e6, None, dev)
    for t in (b, n * sq):
        proj = rnd(t, -(-(heads * (dim + rot) + row + heads) // 64) * 64)        # rows of a PackedLinear
        pos = torch.randint(0, 8192, (t,), device=dev)
        slots = torch.randperm(nblk * bs, device=dev)[:t].to(torch.int32)
        decode = t == b
        qx = rnd(t if decode else 1, heads, row)
        norm = torch.ones(rank, device=dev)
        hbm(f"latent_front, {t} rows", t * 2 * (2 * heads * rot + 2 * row),
            lambda: ho.latent_front(proj, heads, dim, rot, rot, heads * (dim + rot), rank, norm, 1e-6, table, pos, slots, cache, rank, qx, t if decode else 0))
        qkv = rnd(t, (heads + 16) * 128)
        qv, kk, vv = (x.view(t, -1, 128) for x in qkv.split([heads * 128, 8 * 128, 8 * 128], dim=-1))
        kc, w128, cs = rnd(nblk, bs, 8, 128), torch.ones(128, dtype=bf, device=dev), rnd(8192, 128)
        hbm(f"qwen3: norm + rotary + append, {t} rows", t * (2 * heads * 128 * 2 + 4 * 8 * 128 * 2),
            lambda: ops.qk_norm_rope_store_kvcache(qv, kk, vv, pos, w128, w128, 1e-6, cs, kc, kc, slots, write_key=False))
        del kc, qkv, proj
    x, w = rnd(b, heads, dim), rnd(heads, rank, dim)
    y = torch.empty((b, heads, rank), dtype=bf, device=dev)
    hbm("head_matmul W_uk^T q, 64 rows", 2 * (x.numel() + w.numel() + y.numel()), lambda: ho.head_matmul(x, w, y, rank, dim))
    w2 = rnd(heads, vdim, rank)
    hbm("head_matmul W_uv c (gated), 64 rows", 2 * (x.numel() + w2.numel() + y.numel()), lambda: ho.head_matmul(y, w2, x, vdim, rank, gate=gate[:b]))
    wn = rnd(4096, 2048)
    xs = rnd(b, 2048)
    hbm("qwen3: split-K GEMM 64 x 4096 x 2048 (weights of the size of the above, x4)", 2 * wn.numel(), lambda: ops.skinny_linear(xs, wn))
    del cache

    # ---- delta rule
    s = ho.DeltaShape(heads, heads, 128, 128, 4, 1e-6)
    slots_n = 64
    state = torch.zeros(slots_n, heads, 128, 128, device=dev)
    ring = torch.zeros(slots_n, 4, s.channels, dtype=bf, device=dev)
    wts = [torch.randn(s.channels, 4, device=dev) * .5, torch.zeros(heads, device=dev), torch.full((heads * 128,), -3.0, device=dev), torch.ones(128, device=dev)]
    proj, dec, gt = rnd(b, s.channels + heads), rnd(b, heads * 128), rnd(b, heads * 128)
    o2 = torch.empty((b, heads * 128), dtype=bf, device=dev)
    pos = torch.full((b,), 77, dtype=torch.int64, device=dev)
    sl = torch.arange(b, dtype=torch.int32, device=dev)
    hbm("delta_step, 64 sequences", 2 * state.numel() * 4 + 2 * (proj.numel() + dec.numel() + gt.numel() + 5 * s.channels // 3 * b),
        lambda: ho.delta_step(s, proj, s.channels, dec, gt, *wts, ring, state, sl, pos, o2))
    for n, sq in ((1, 2048), (8, 2048)):
        t = n * sq
        proj, dec, gt = rnd(t, s.channels + heads), rnd(t, heads * 128), rnd(t, heads * 128)
        o3 = torch.empty((t, heads * 128), dtype=bf, device=dev)
        per = sq // CHUNK
        portions = torch.tensor([(i * per, per, i, 0) for i in range(n)], dtype=torch.int32, device=dev)
        chunks = torch.tensor([(i * sq + r, CHUNK, r, 0, i, 0) for i in range(n) for r in range(0, sq, CHUNK)], dtype=torch.int32, device=dev)
        rs = torch.tensor([(i, sq - 1 - r) for i in range(n) for r in range(sq)], dtype=torch.int32, device=dev)
        pos = torch.arange(sq, device=dev).repeat(n)
        # three products with the [128, 128] state and two inside the chunk, per token and head
        mfma(f"delta_chunks, {n} x {sq}", t * heads * (6 * 128 * 128 + 4 * 16 * 128), F32_MFMA_PEAK_TFLOPS,
             lambda: ho.delta_chunks(s, proj, s.channels, dec, gt, *wts, ring, state, portions, chunks, rs, pos, 0, o3),
             "all three launches, against the float32 matrix peak")
    del proj, dec, gt

    # ---- residual stream and activation
    for t in (b, 16384):
        x32, y = rnd(t, width, dtype=torch.float32), rnd(t, width)
        w32, wb = torch.ones(width, device=dev), torch.ones(width, dtype=bf, device=dev)
        hbm(f"residual_norm, {t} rows", t * width * (4 + 4 + 2 + 2), lambda: ho.residual_norm(x32, 1e-6, y=y, w_post=w32, w_pre=w32))
        res = rnd(t, width)
        hbm(f"qwen3: rms_norm with residual, {t} rows", t * width * 8, lambda: ops.rms_norm(y, wb, 1e-6, res))
        gu = rnd(t, 2 * ff)
        act = torch.empty((t, ff), dtype=bf, device=dev)
        hbm(f"gelu_tanh_and_mul, {t} rows", t * ff * 6, lambda: ho.gelu_tanh_and_mul(gu))
        hbm(f"qwen3: silu_and_mul, {t} rows", t * ff * 6, lambda: ops.silu_and_mul(act, gu))
    return out


def vokelix_kernels(heads=32, kv_heads=8, width=4096, ff=12288):
    """Every kernel of Vokelix at the sizes of an 8B model's layers, with what bounds it, beside the like kernel of Qwen3
    (attention, norms, activation) or Merilorn (recurrence) at the same sizes.  Buffers are larger than the caches or
    rotated, where a kernel's bytes would fit them."""
    from infer_amd import hybrid_ops as ho, ops, workloads
    from infer_amd.layers import yarn_rotary_table
    from infer_amd.step_plan import CHUNK
    dev, bf = torch.device("cuda:0"), torch.bfloat16
    out, rnd, hbm, mfma = roofline_table(dev)
    d, n, sq = 128, 8, 2048
    rows = n * sq

    # ---- decode attention
    bs = 256
    for b, ctx in ((64, 4096), (64, 1024), (16, 4096)):
        nblk = b * ctx // bs
        cache = rnd(nblk, kv_heads, bs, 2 * d)
        tables = torch.randperm(nblk, device=dev).to(torch.int32).view(b, -1)
        lens = torch.full((b,), ctx, dtype=torch.int32, device=dev)
        qx, gate, sink, o = rnd(b, heads, d), rnd(b, heads), torch.randn(heads, device=dev), torch.empty((b, heads * d), dtype=bf, device=dev)
        hbm(f"grouped_attention decode, {b} x {ctx}", b * ctx * kv_heads * 2 * d * 2,
            lambda: ho.grouped_attention(qx, cache, tables, lens, 0.09, d, o, sink, gate))
        wl = workloads.make_decode_workload("point", [ctx] * b, heads, kv_heads, seed=0, q_scale=d ** -0.5, device=dev, device_fill=True)
        o3 = torch.empty((b, heads, d), dtype=bf, device=dev)
        hbm(f"qwen3: paged decode attention, {b} x {ctx}", wl.decode_bytes,
            lambda: ops.paged_attn_decode(wl.q, wl.k_cache, wl.v_cache, wl.block_table, wl.context_lens, wl.scale, o3))
        del wl, cache

    # ---- prefill attention
    cu = torch.arange(0, n + 1, dtype=torch.int32, device=dev) * sq
    nblk = rows // bs
    cache = rnd(nblk, kv_heads, bs, 2 * d)
    tables = torch.randperm(nblk, device=dev).to(torch.int32).view(n, -1)
    seqs = torch.arange(n, dtype=torch.int32, device=dev)
    hbm(f"grouped_gather, {rows} rows", 2 * cache.numel() * 2, lambda: ho.grouped_gather(cache, tables, seqs, cu, rows, sq))
    kv = ho.grouped_gather(cache, tables, seqs, cu, rows, sq)
    proj, at, sink = rnd(rows, (heads + 2 * kv_heads) * d + 64), torch.empty((rows, heads * d), dtype=bf, device=dev), torch.randn(heads, device=dev)
    pairs = n * sq * (sq + 1) // 2
    mfma("grouped_prefill, 8 x 2048", 4 * heads * d * pairs, BF16_PEAK_TFLOPS,
         lambda: ho.grouped_prefill(proj, kv[:, :, d:], kv[:, :, :d], sink, proj[:, -heads:], at, cu, cu, sq, heads, d, d, 0.09))
    q3, k3 = rnd(rows, heads, d), rnd(rows, kv_heads, d)
    mfma("qwen3: prefill attention, 8 x 2048", 4 * heads * d * pairs, BF16_PEAK_TFLOPS,
         lambda: ops.flash_attn_varlen_func(q3, k3, k3, max_seqlen_q=sq, cu_seqlens_q=cu, max_seqlen_k=sq, cu_seqlens_k=cu))
    del q3, k3, kv

    # ---- front end
    table = yarn_rotary_table(64, 8192, 1e6, None, dev)
    for t in (64, rows):
        pos = torch.randint(0, 8192, (t,), device=dev)
        slots = torch.randperm(nblk * bs, device=dev)[:t].to(torch.int32)
        x = proj[:t]
        bias, qn, kn = (torch.randn(c, device=dev) for c in (proj.shape[1], heads * d, kv_heads * d))
        qx = rnd(t if t == 64 else 1, heads, d)
        moved = t * 2 * (2 * heads + 4 * kv_heads) * d
        hbm(f"grouped_front, {t} rows", moved, lambda: ho.grouped_front(
            x, heads, kv_heads, d, d, heads * d, (heads + kv_heads) * d, bias, qn, kn, 1e-6, table, 64, pos, slots, cache, d, d, qx, t if t == 64 else 0))
        qkv = rnd(t, (heads + 2 * kv_heads) * d)
        qv, kk, vv = (y.view(t, -1, d) for y in qkv.split([heads * d, kv_heads * d, kv_heads * d], dim=-1))
        kc, w128, cs = rnd(nblk, bs, kv_heads, d), torch.ones(d, dtype=bf, device=dev), rnd(8192, d)
        hbm(f"qwen3: norm + rotary + append, {t} rows", moved,
            lambda: ops.qk_norm_rope_store_kvcache(qv, kk, vv, pos, w128, w128, 1e-6, cs, kc, kc, slots, write_key=False))
        del kc, qkv
    del proj, at, cache

    # ---- linear attention
    state = torch.zeros(64, heads, d, d, device=dev)
    hd = heads * d
    decay = ho.decay_constants([1.0 - 2.0 ** (-4.0 - 7.0 * h / heads) for h in range(heads)], dev)
    table = yarn_rotary_table(d, 8192, 1e4, None, dev)
    kinds = {"lightning": (ho.DecayShape(heads, d, d, 1e-6, True, 0, 1.0, False, False), None, torch.ones(hd, device=dev)),
             "retention": (ho.DecayShape(heads, d, d, 1e-6, False, d, d ** -0.5, True, True), table, None)}
    sl, pos = torch.arange(64, dtype=torch.int32, device=dev), torch.full((64,), 77, dtype=torch.int64, device=dev)
    off = [0, hd, 2 * hd, 3 * hd]
    x, o2 = rnd(64, 4 * hd), torch.empty((64, hd), dtype=bf, device=dev)
    for kind, (s, tab, norm) in kinds.items():
        hbm(f"decay_attention ({kind}), one token x 64", 2 * state.numel() * 4 + 5 * 64 * hd * 2,
            lambda: ho.decay_attention(s, x, off, decay, tab, norm, state, sl, pos, 64, None, 0, o2))
    for m, length in ((1, 2048), (8, 2048), (1, 16384)):
        t = m * length
        x, o2 = rnd(t, 4 * hd), torch.empty((t, hd), dtype=bf, device=dev)
        spans = torch.tensor([(i * length, length, i, 0) for i in range(m)], dtype=torch.int32, device=dev)
        for kind, (s, tab, norm) in kinds.items():
            tab = yarn_rotary_table(d, 16384, 1e4, None, dev) if tab is not None else None
            hbm(f"decay_attention ({kind}), {m} x {length}", 5 * t * hd * 2,
                lambda: ho.decay_attention(s, x, off, decay, tab, norm, state, None, None, 0, spans, length, o2), "all launches; q, k, v, gate, result")
    del x
    s = ho.DeltaShape(heads, heads, d, d, 4, 1e-6)
    ring = torch.zeros(64, 4, s.channels, dtype=bf, device=dev)
    wts = [torch.randn(s.channels, 4, device=dev) * .5, torch.zeros(heads, device=dev), torch.full((hd,), -3.0, device=dev), torch.ones(d, device=dev)]
    x, dec, gt = rnd(64, s.channels + heads), rnd(64, hd), rnd(64, hd)
    o2 = torch.empty((64, hd), dtype=bf, device=dev)
    hbm("merilorn: delta_step, one token x 64", 2 * state.numel() * 4 + 2 * (x.numel() + 3 * dec.numel() + 5 * s.channels // 3 * 64),
        lambda: ho.delta_step(s, x, s.channels, dec, gt, *wts, ring, state, sl, pos, o2))
    for m in (1, 8):
        t = m * sq
        x, dec, gt, o2 = rnd(t, s.channels + heads), rnd(t, hd), rnd(t, hd), torch.empty((t, hd), dtype=bf, device=dev)
        per = sq // CHUNK
        portions = torch.tensor([(i * per, per, i, 0) for i in range(m)], dtype=torch.int32, device=dev)
        chunks = torch.tensor([(i * sq + r, CHUNK, r, 0, i, 0) for i in range(m) for r in range(0, sq, CHUNK)], dtype=torch.int32, device=dev)
        rs = torch.tensor([(i, sq - 1 - r) for i in range(m) for r in range(sq)], dtype=torch.int32, device=dev)
        pos = torch.arange(sq, device=dev).repeat(m)
        mfma(f"merilorn: delta_chunks, {m} x {sq}", t * heads * (6 * d * d + 4 * 16 * d), F32_MFMA_PEAK_TFLOPS,
             lambda: ho.delta_chunks(s, x, s.channels, dec, gt, *wts, ring, state, portions, chunks, rs, pos, 0, o2))
        us = out[f"merilorn: delta_chunks, {m} x {sq}"]["us"]
        out[f"merilorn: delta_chunks, {m} x {sq}"]["note"] = "frac: of the float32 matrix peak; of the memory bandwidth: %.3f" % (
            6 * t * hd * 2 / us / 1e3 / HBM_PEAK_GBS)
    del x, dec, gt

    # ---- residual stream and activation
    for t in (64, rows):
        x32, y, w32, wb = rnd(t, width, dtype=torch.float32), rnd(t, width), torch.ones(width, device=dev), torch.ones(width, dtype=bf, device=dev)
        hbm(f"post_norm, {t} rows", t * width * 12, lambda: ho.post_norm(x32, 1e-6, y=y, w_post=w32, alpha=2.0))
        hbm(f"merilorn: residual_norm, {t} rows", t * width * 12, lambda: ho.residual_norm(x32, 1e-6, y=y, w_post=w32, w_pre=w32))
        res = rnd(t, width)
        hbm(f"qwen3: rms_norm with residual, {t} rows", t * width * 8, lambda: ops.rms_norm(y, wb, 1e-6, res))
        gu = rnd(t, 2 * ff)
        act = torch.empty((t, ff), dtype=bf, device=dev)
        hbm(f"silu_and_mul, {t} rows", t * ff * 6, lambda: ho.silu_and_mul(gu))
        hbm(f"qwen3: silu_and_mul, {t} rows", t * ff * 6, lambda: ops.silu_and_mul(act, gu))
    return out


def dogetar_kernels(heads=32, kv_heads=8, width=4096, ff=12288):
    """Every kernel of Dogetar at the sizes of an 8B model's layers, with what bounds it, beside the like kernel of Qwen3 (attention, norms,
    products) or Vokelix (recurrence, residual, activation) at the same sizes."""
    from infer_amd import hybrid_ops as ho, ops, workloads
    from infer_amd.layers import banded_rotary_table
    dev, bf = torch.device("cuda:0"), torch.bfloat16
    out, rnd, hbm, mfma = roofline_table(dev)
    d, n, sq, bs = 128, 8, 2048, 256
    rows = n * sq

    def shape(maps=1, mask="window", size=1 << 20, bias=False):
        return ho.MaskedShape(heads, kv_heads, d // maps, d, 0.09, maps=maps, mask=mask, mask_size=size, distance_bias=bias, lam=0.4, eps=1e-6,
                              rot_dims=64)

    # ---- decode attention: b sequences of which every query sees `seen` keys
    gate, sink = rnd(64, heads), torch.randn(heads, device=dev)
    for b, seen in ((64, 4096), (64, 1024), (16, 4096)):
        nblk = b * 4096 // bs
        cache = rnd(nblk, kv_heads, bs, 2 * d)
        tables = torch.randperm(nblk, device=dev).to(torch.int32).view(b, -1)
        lens, o = torch.full((b,), 4096, dtype=torch.int32, device=dev), torch.empty((b, heads * d), dtype=bf, device=dev)
        for name, s, extra in (("window", shape(size=seen), (None, None)), ("chunk, bias, sink", shape(1, "chunk", seen, True), (sink, None)),
                               ("chunk, two maps, gate", shape(2, "chunk", seen), (None, gate[:b]))):
            qx = rnd(b, heads * s.maps, s.key_pad)
            hbm(f"masked_attention decode ({name}), {b} x {seen}", b * seen * kv_heads * 2 * d * 2,
                lambda: ho.masked_attention(s, qx, cache, tables, lens, o, *extra, max_keys=4096))
        wl = workloads.make_decode_workload("point", [seen] * b, heads, kv_heads, seed=0, q_scale=d ** -0.5, device=dev, device_fill=True)
        o3 = torch.empty((b, heads, d), dtype=bf, device=dev)
        hbm(f"qwen3: paged decode attention, {b} x {seen}", wl.decode_bytes,
            lambda: ops.paged_attn_decode(wl.q, wl.k_cache, wl.v_cache, wl.block_table, wl.context_lens, wl.scale, o3))
        del wl, cache

    # ---- prefill attention
    cu = torch.arange(0, n + 1, dtype=torch.int32, device=dev) * sq
    nblk = rows // bs
    cache = rnd(nblk, kv_heads, bs, 2 * d)
    tables = torch.randperm(nblk, device=dev).to(torch.int32).view(n, -1)
    seqs = torch.arange(n, dtype=torch.int32, device=dev)
    hbm(f"masked_gather, {rows} rows", 2 * cache.numel() * 2, lambda: ho.masked_gather(shape(), cache, tables, seqs, cu, cu, rows, sq))
    kv = ho.masked_gather(shape(), cache, tables, seqs, cu, cu, rows, sq)
    proj, at = rnd(rows, (heads + 2 * kv_heads) * d + 64), torch.empty((rows, heads * d), dtype=bf, device=dev)
    triangle, half = sq * (sq + 1) // 2, sq // 2
    for name, s, pairs, extra in (("window", shape(), triangle, (None, None)), ("chunk, bias, sink", shape(1, "chunk", sq, True), triangle, (sink, None)),
                                  ("chunk, two maps, gate", shape(2, "chunk", sq), triangle, (None, proj[:, -heads:])),
                                  ("window of 1024", shape(size=half), triangle - half * (half + 1) // 2, (None, None)),
                                  ("chunks of 1024, two maps", shape(2, "chunk", half), half * (half + 1), (None, None))):
        # two maps: two products of half as many entries with the keys, two with the values
        mfma(f"masked_prefill ({name}), 8 x 2048", 2 * heads * d * (1 + s.maps) * n * pairs, BF16_PEAK_TFLOPS,
             lambda: ho.masked_prefill(s, proj, kv, at, cu, cu, sq, *extra))
    q3, k3 = rnd(rows, heads, d), rnd(rows, kv_heads, d)
    mfma("qwen3: prefill attention, 8 x 2048", 4 * heads * d * n * triangle, BF16_PEAK_TFLOPS,
         lambda: ops.flash_attn_varlen_func(q3, k3, k3, max_seqlen_q=sq, cu_seqlens_q=cu, max_seqlen_k=sq, cu_seqlens_k=cu))
    zero = torch.zeros(rows, heads, dtype=bf, device=dev)
    mfma("vokelix: grouped_prefill, 8 x 2048", 4 * heads * d * n * triangle, BF16_PEAK_TFLOPS,
         lambda: ho.grouped_prefill(proj, kv[:, :, d:], kv[:, :, :d], sink, zero, at, cu, cu, sq, heads, d, d, 0.09))
    del q3, k3, kv, zero

    # ---- front end
    table = banded_rotary_table(64, 8192, 1e6, None, dev)
    for t in (64, rows):
        pos, slots = torch.randint(0, 8192, (t,), device=dev), torch.randperm(nblk * bs, device=dev)[:t].to(torch.int32)
        x, bias = proj[:t], torch.randn(proj.shape[1], device=dev)
        moved = t * 2 * (2 * heads + 4 * kv_heads) * d
        for name, s, extra in (("bias, norm", shape(), (bias, torch.ones(d, device=dev), torch.ones(d, device=dev))),
                               ("two maps", shape(2), (None, None, None))):
            split = t if t == 64 else 0
            qx = rnd(max(split, 1), heads * s.maps, s.key_pad)
            hbm(f"head_front ({name}), {t} rows", moved + split * 2 * heads * d * (s.maps - 1),
                lambda: ho.head_front(s, x, [0, heads * d, (heads + kv_heads) * d], *extra, table, pos, slots, cache, qx, split))
        qkv = rnd(t, (heads + 2 * kv_heads) * d)
        qv, kk, vv = (y.view(t, -1, d) for y in qkv.split([heads * d, kv_heads * d, kv_heads * d], dim=-1))
        kc, w128, cs = rnd(nblk, bs, kv_heads, d), torch.ones(d, dtype=bf, device=dev), rnd(8192, d)
        hbm(f"qwen3: norm + rotary + append, {t} rows", moved,
            lambda: ops.qk_norm_rope_store_kvcache(qv, kk, vv, pos, w128, w128, 1e-6, cs, kc, kc, slots, write_key=False))
        del kc, qkv
    del proj, at, cache

    # ---- recurrence
    s = ho.StateSpaceShape(2 * heads, 64, 128, 2, 4, 2, 1e-6)
    hd, cols = s.inner, 2 * s.inner + 2 * s.groups * s.state + 2 * heads
    cols = -(-cols // 64) * 64
    state, ring = torch.zeros(64, s.heads, s.state, s.vdim, device=dev), torch.zeros(64, 4, s.channels, dtype=bf, device=dev)
    wts = [torch.randn(s.channels, 4, device=dev) * .5, torch.zeros(s.channels, device=dev), torch.zeros(s.heads, device=dev),
           torch.zeros(s.heads, device=dev), torch.ones(s.heads, device=dev), torch.ones(hd, device=dev)]
    off, sl, pos = (0, hd, hd + s.channels), torch.arange(64, dtype=torch.int32, device=dev), torch.full((64,), 77, dtype=torch.int64, device=dev)
    x, o2 = rnd(64, cols), torch.empty((64, hd), dtype=bf, device=dev)
    hbm("state_space, one token x 64", 2 * state.numel() * 4 + 64 * 2 * (2 * hd + 4 * s.channels),
        lambda: ho.state_space(s, x, off, *wts, ring, state, sl, pos, 64, None, 0, None, o2))
    dec = ho.DecayShape(heads, d, d, 1e-6, True, 0, 1.0, False, False)
    decay = ho.decay_constants([1.0 - 2.0 ** (-4.0 - 7.0 * h / heads) for h in range(heads)], dev)
    dstate, dnorm, doff = torch.zeros(64, heads, d, d, device=dev), torch.ones(heads * d, device=dev), [i * heads * d for i in range(4)]
    x4 = rnd(64, 4 * heads * d)
    hbm("vokelix: decay_attention (lightning), one token x 64", 2 * dstate.numel() * 4 + 5 * 64 * heads * d * 2,
        lambda: ho.decay_attention(dec, x4, doff, decay, None, dnorm, dstate, sl, pos, 64, None, 0, o2))
    for m, length in ((1, 2048), (8, 2048), (1, 16384)):
        t = m * length
        x, o2, x4 = rnd(t, cols), torch.empty((t, hd), dtype=bf, device=dev), rnd(t, 4 * heads * d)
        spans = torch.tensor([(i * length, length, i, 0) for i in range(m)], dtype=torch.int32, device=dev)
        rs = torch.stack((torch.arange(m, device=dev).repeat_interleave(length), torch.arange(length - 1, -1, -1, device=dev).repeat(m)), 1).to(torch.int32)
        pos = torch.arange(length, device=dev).repeat(m)
        hbm(f"state_space, {m} x {length}", t * 2 * (2 * hd + s.channels + s.heads),
            lambda: ho.state_space(s, x, off, *wts, ring, state, None, pos, 0, spans, length, rs, o2), "all launches; z, x, B, C, dt, result")
        hbm(f"vokelix: decay_attention (lightning), {m} x {length}", 5 * t * heads * d * 2,
            lambda: ho.decay_attention(dec, x4, doff, decay, None, dnorm, dstate, None, None, 0, spans, length, o2), "all launches; q, k, v, gate, result")
    del x, x4, state, dstate

    # ---- mixture of experts, and products of the same numbers as dense ones
    experts, top, eff = 16, 4, ff // 4
    ms = ho.MoeShape(width, eff, experts, top, 0, 4, 2, 1.0)
    wr, wu, wd = rnd(experts, width), rnd(experts, 2 * eff, width), rnd(experts, width, eff)
    counts, corr = torch.zeros(experts, dtype=torch.int32, device=dev), torch.zeros(experts, device=dev)
    du, dd = rnd(2 * eff * top, width), rnd(width, eff * top)
    for t in (16, 64, rows):
        h = rnd(t, width) * 0.05
        if t < rows:
            weights = 3 * eff * width * 2
            r = ho.moe(ms, h, wr, corr, wu, wd, counts)
            used = int((torch.bincount((wr.float() @ h.float().T).topk(top, 0).indices.flatten(), minlength=experts) > 0).sum())
            places = r.rows.shape[0]
            hbm(f"moe, {t} rows", weights * experts + places * 2 * (2 * width + 2 * eff), lambda: ho.moe(ms, h, wr, corr, wu, wd, counts),
                f"all launches: routing, sort, two products; weights of all experts ({used} of {experts} chosen without groups)")
            act = rnd(t, eff * top)
            hbm(f"qwen3: two dense products of as many columns per row, {t} rows", weights * top, lambda: (ops.linear(h, du), ops.linear(act, dd)))
        else:
            mfma(f"moe, {t} rows", 2 * t * top * 3 * eff * width, BF16_PEAK_TFLOPS, lambda: ho.moe(ms, h, wr, corr, wu, wd, counts),
                 "all launches: routing, sort, two products")
            act = rnd(t, eff * top)
            mfma(f"qwen3: two dense products of as many columns per row, {t} rows", 2 * t * top * 3 * eff * width, BF16_PEAK_TFLOPS,
                 lambda: (torch.nn.functional.linear(h, du), torch.nn.functional.linear(act, dd)), "vendor GEMM")
        r = ho.moe(ms, h, wr, corr, wu, wd, counts)
        x32, w32, y = rnd(t, width, dtype=torch.float32), torch.ones(width, device=dev), rnd(t, width)
        hbm(f"pre_norm, {t} rows", t * width * 12, lambda: ho.pre_norm(x32, w32, 1e-6, y=y, scale=w32))
        r.shared = y
        hbm(f"pre_norm with {top} experts, {t} rows", t * width * (12 + 2 * top), lambda: ho.pre_norm(x32, w32, 1e-6, y=r, scale=w32))
        hbm(f"vokelix: post_norm, {t} rows", t * width * 12, lambda: ho.post_norm(x32, 1e-6, y=y, w_post=w32, alpha=1.0))
        gu = rnd(t, 2 * ff)
        hbm(f"clamped_gate_and_mul, {t} rows", t * ff * 6, lambda: ho.clamped_gate_and_mul(gu, 7.0))
        hbm(f"vokelix: silu_and_mul, {t} rows", t * ff * 6, lambda: ho.silu_and_mul(gu))
        del r, gu, act
    logits = rnd(64, 151936)
    hbm("softcap, 64 rows of 151936", logits.numel() * 6, lambda: ho.softcap(logits, 30.0))
    return out


def tulurax_kernels(width=4096, ff=18432):
    """Every kernel of Tulurax at the sizes of an 8B model's layers, with what bounds it, beside the like kernel of Vokelix (attention,
    recurrence, residual, activation) or Qwen3 (attention) at the same sizes."""
    from infer_amd import hybrid_ops as ho, ops, workloads
    from infer_amd.layers import yarn_rotary_table
    dev, bf = torch.device("cuda:0"), torch.bfloat16
    out, rnd, hbm, mfma = roofline_table(dev)
    d, n, sq, bs, kv_heads = 128, 8, 2048, 256, 8
    rows = n * sq

    # ---- decode attention
    for heads in (16, 32):
        s = ho.TalkShape(heads, kv_heads, d, d, 0.09, 1e-6)
        talk, sink = rnd(heads, heads), torch.randn(heads, device=dev)
        for b, seen in ((64, 4096), (64, 1024), (16, 4096)):
            nblk = b * seen // bs
            keys, values = rnd(nblk, kv_heads, bs // 32, d // 8, 32, 8), rnd(nblk, kv_heads, bs // 32, d // 16, 4, 16, 8)
            tables = torch.randperm(nblk, device=dev).to(torch.int32).view(b, -1)
            lens, o, qx = torch.full((b,), seen, dtype=torch.int32, device=dev), torch.empty((b, heads * d), dtype=bf, device=dev), rnd(b, heads, d)
            moved = b * seen * kv_heads * 2 * d * 2
            hbm(f"talking_attention decode, {heads} heads, {b} x {seen}", moved,
                lambda: ho.talking_attention(s, qx, keys, values, talk, tables, lens, o), "all launches; keys and values")
            cache = rnd(nblk, kv_heads, bs, 2 * d)
            hbm(f"vokelix: grouped_attention decode, {heads} heads, {b} x {seen}", moved,
                lambda: ho.grouped_attention(qx, cache, tables, lens, 0.09, d, o, sink, qx[:, :, 0].contiguous()))
            del cache, keys, values
            wl = workloads.make_decode_workload("point", [seen] * b, heads, kv_heads, seed=0, q_scale=d ** -0.5, device=dev, device_fill=True)
            o3 = torch.empty((b, heads, d), dtype=bf, device=dev)
            hbm(f"qwen3: paged decode attention, {heads} heads, {b} x {seen}", wl.decode_bytes,
                lambda: ops.paged_attn_decode(wl.q, wl.k_cache, wl.v_cache, wl.block_table, wl.context_lens, wl.scale, o3))
            del wl

    # ---- prefill attention
    triangle = sq * (sq + 1) // 2
    nblk = rows // bs
    for m, length in ((8, 2048), (1, 16384), (1, 2048)):
        t, blocks = m * length, m * length // bs
        cu = torch.arange(0, m + 1, dtype=torch.int32, device=dev) * length
        tables = torch.randperm(blocks, device=dev).to(torch.int32).view(m, -1)
        seqs, pairs = torch.arange(m, dtype=torch.int32, device=dev), m * length * (length + 1) // 2
        for heads, kv in ((16, 8), (16, 16), (32, 8)) if m == 8 else ((16, 8),):
            s = ho.TalkShape(heads, kv, d, d, 0.09, 1e-6)
            talk, q, at = rnd(heads, heads), rnd(t, heads * d), torch.empty((t, heads * d), dtype=bf, device=dev)
            keys, values = rnd(blocks, kv, bs // 32, d // 8, 32, 8), rnd(blocks, kv, bs // 32, d // 16, 4, 16, 8)
            mfma(f"talking_prefill, {heads} heads of {kv} keys, {m} x {length}", (4 * heads * d + 2 * heads * heads) * pairs, BF16_PEAK_TFLOPS,
                 lambda: ho.talking_prefill(s, q, keys, values, talk, tables, seqs, cu, cu, length, length, at,
                                            max_score=s.max_score(length)),
                 "both launches; each product counted once")
            dense = rnd(t, kv, 2 * d)
            zero, sink = torch.zeros(t, heads, dtype=bf, device=dev), torch.zeros(heads, device=dev)
            mfma(f"vokelix: grouped_prefill, {heads} heads of {kv} keys, {m} x {length}", 4 * heads * d * pairs, BF16_PEAK_TFLOPS,
                 lambda: ho.grouped_prefill(q, dense[:, :, d:], dense[:, :, :d], sink, zero, at, cu, cu, length, heads, d, d, 0.09))
            del dense, zero
            if heads > kv:
                q3, k3 = q.view(t, heads, d), rnd(t, kv, d)
                mfma(f"qwen3: prefill attention, {heads} heads of {kv} keys, {m} x {length}", 4 * heads * d * pairs, BF16_PEAK_TFLOPS,
                     lambda: ops.flash_attn_varlen_func(q3, k3, k3, max_seqlen_q=length, cu_seqlens_q=cu, max_seqlen_k=length, cu_seqlens_k=cu))
                del q3, k3
            del q, at, keys, values

    # ---- front end
    heads = 16
    s = ho.TalkShape(heads, kv_heads, d, d, 0.09, 1e-6, True, 0.1, 8192)
    keys, values = rnd(nblk, kv_heads, bs // 32, d // 8, 32, 8), rnd(nblk, kv_heads, bs // 32, d // 16, 4, 16, 8)
    cache = rnd(nblk, kv_heads, bs, 2 * d)
    table, ones = yarn_rotary_table(64, 8192, 1e6, None, dev), torch.ones(heads * d, device=dev)
    for t in (64, rows):
        pos, slots = torch.randint(0, 8192, (t,), device=dev), torch.arange(t, device=dev, dtype=torch.int32)
        x, split = rnd(t, (heads + 2 * kv_heads) * d), t if t == 64 else 0
        qx, moved = rnd(max(split, 1), heads, d), t * 2 * (2 * heads + 4 * kv_heads) * d
        hbm(f"unit_head_front, {t} rows", moved,
            lambda: ho.unit_head_front(s, x, [0, heads * d, (heads + kv_heads) * d], pos, slots, keys, values, qx, split))
        hbm(f"vokelix: grouped_front, {t} rows", moved,
            lambda: ho.grouped_front(x, heads, kv_heads, d, d, heads * d, (heads + kv_heads) * d, torch.zeros(x.shape[1], device=dev), ones, ones[:kv_heads * d].contiguous(),
                                     1e-6, table, 64, pos, slots, cache, d, d, qx, split))
    del keys, values, cache

    # ---- retention, without and with rotation
    decay = ho.decay_constants([1.0 - 2.0 ** (-4.0 - 7.0 * h / heads) for h in range(heads)], dev)
    plain, turned = (ho.DecayShape(heads, d, d, 1e-6, False, rot, d ** -0.5, True, True) for rot in (0, d))
    wide = yarn_rotary_table(d, 16384, 1e4, None, dev)
    state, gain, off = torch.zeros(64, heads, d, d, device=dev), torch.full((heads * d,), 0.7, device=dev), [i * heads * d for i in range(4)]
    sl, pos = torch.arange(64, dtype=torch.int32, device=dev), torch.full((64,), 77, dtype=torch.int64, device=dev)
    x, o2 = rnd(64, 4 * heads * d), torch.empty((64, heads * d), dtype=bf, device=dev)
    for name, shape, tab, norm in (("", plain, None, gain), ("vokelix: ", turned, wide, None)):
        hbm(f"{name}decay_attention (retention), one token x 64", 2 * state.numel() * 4 + 5 * 64 * heads * d * 2,
            lambda: ho.decay_attention(shape, x, off, decay, tab, norm, state, sl, pos, 64, None, 0, o2))
    for m, length in ((1, 2048), (8, 2048), (1, 16384)):
        t = m * length
        x, o2 = rnd(t, 4 * heads * d), torch.empty((t, heads * d), dtype=bf, device=dev)
        spans = torch.tensor([(i * length, length, i, 0) for i in range(m)], dtype=torch.int32, device=dev)
        for name, shape, tab, norm in (("", plain, None, gain), ("vokelix: ", turned, wide, None)):
            hbm(f"{name}decay_attention (retention), {m} x {length}", 5 * t * heads * d * 2,
                lambda: ho.decay_attention(shape, x, off, decay, tab, norm, state, None, None, 0, spans, length, o2),
                "all launches; q, k, v, gate, result")
    del x, state

    # ---- residual stream, activation, logits
    for t in (64, rows):
        x32, w32, y = rnd(t, width, dtype=torch.float32), torch.ones(width, device=dev), rnd(t, width)
        norm = ho.TanhNorm(0.5, w32, w32)
        hbm(f"tanh_norm with a bias, {t} rows", t * width * 12, lambda: ho.tanh_norm(x32, norm, y=y, bias=w32))
        hbm(f"vokelix: post_norm, {t} rows", t * width * 12, lambda: ho.post_norm(x32, 1e-6, y=y, w_post=w32, alpha=1.0))
        up, bias = rnd(t, ff), torch.zeros(ff, device=dev)
        hbm(f"xielu, {t} rows", t * ff * 4, lambda: ho.xielu(up, bias, 0.8, 1.2))
        gu = rnd(t, ff // 3 * 4)
        hbm(f"vokelix: silu_and_mul, {t} rows", t * ff // 3 * 2 * 6, lambda: ho.silu_and_mul(gu))
        del gu, up, x32
    logits = rnd(64, 151936)
    hbm("softcap, 64 rows of 151936", logits.numel() * 6, lambda: ho.softcap(logits, 30.0, 2.0))
    return out


def engine_points(models):
    points = []
    for size, batch, prompt, new in (("0.6b", 64, 1024, 64), ("8b", 64, 1024, 64), ("8b", 16, 4096, 64)):
        for model in models:
            points.append(hybrid_engine_point(size, model, batch, prompt, new))
            print(points[-1], file=sys.stderr, flush=True)
    return points


def run_hybrid(args):
    """Merilorn beside Qwen3 at equal width, feed-forward, heads and number of layers: the engine's prefill and
    decode throughput, then the kernels one by one."""
    points = [] if args.hybrid_kernels_only else engine_points(("merilorn", "qwen3"))
    print(json.dumps({"hybrid_engine": points, "hybrid_kernels": hybrid_kernels()}))


def run_vokelix(args):
    """Vokelix beside Qwen3 and Merilorn, as ``run_hybrid``."""
    points = [] if args.hybrid_kernels_only else engine_points(("vokelix", "qwen3", "merilorn"))
    print(json.dumps({"vokelix_engine": points, "vokelix_kernels": vokelix_kernels()}))


def run_dogetar(args):
    """Dogetar beside Qwen3 and Vokelix, as ``run_hybrid``."""
    points = [] if args.hybrid_kernels_only else engine_points(("dogetar", "qwen3", "vokelix"))
    print(json.dumps({"dogetar_engine": points, "dogetar_kernels": dogetar_kernels()}))


def run_tulurax(args):
    """Tulurax beside Qwen3 and Vokelix, as ``run_hybrid``."""
    points = [] if args.hybrid_kernels_only else engine_points(("tulurax", "qwen3", "vokelix"))
    print(json.dumps({"tulurax_engine": points, "tulurax_kernels": tulurax_kernels()}))


# ------------------------------------------------------------------------------------------ decode curve
def decode_point(name, wl, copies, iters, splits=0, uniform_len=None):
    """Decode op (split + merge) of one workload, timed as replays of a HIP graph that holds ``copies``
    consecutive steps, each over its own copy of the caches (no host time between launches, reads
    come from HBM).  With ``uniform_len`` the batch's common length is also timed as a host integer
    (``cache_seqlens: int``), the form in which the library may run one kernel without a merge."""
    from infer_amd import ops
    dev = wl.q.device
    b, hq, hkv, d = len(wl.lengths), wl.num_q_heads, wl.num_kv_heads, wl.head_dim
    ks = [wl.k_cache] + [torch.randn_like(wl.k_cache) for _ in range(copies - 1)]
    vs = [wl.v_cache] + [torch.randn_like(wl.v_cache) for _ in range(copies - 1)]
    out = torch.empty((b, hq, d), dtype=torch.bfloat16, device=dev)
    ws = ops.decode_workspace(dev, b, hq, hkv, d)

    def timed(lengths):
        def steps():
            for i in range(copies):
                ops.paged_attn_decode(wl.q, ks[i], vs[i], wl.block_table, lengths, wl.scale, out, ws,
                                      split_workgroups=splits)
        steps()
        torch.cuda.synchronize()
        side = torch.cuda.Stream()
        graph = torch.cuda.CUDAGraph()
        with torch.cuda.stream(side):
            steps()
            side.synchronize()
            with torch.cuda.graph(graph, stream=side):
                steps()
        torch.cuda.synchronize()
        t_spin = time.perf_counter()              # untimed: back to steady clocks after the idle set-up
        while time.perf_counter() - t_spin < 0.03:
            for _ in range(10):
                graph.replay()
            torch.cuda.synchronize()
        return gpu_time_ms(graph.replay, iters, 2) / copies

    nbytes = wl.decode_bytes

    def figures(ms):
        return {"op_us": round(ms * 1e3, 2), "GBps": round(nbytes / ms / 1e6, 1),
                "frac_of_8TBps": round(nbytes / ms / 1e6 / HBM_PEAK_GBS, 4)}

    point = {"name": name, "batch": b, "Hq": hq, "tokens": sum(wl.lengths), "algorithmic_bytes": nbytes,
             **figures(timed(wl.context_lens)), "cache_copies": copies}
    if uniform_len is not None:
        assert all(n == uniform_len for n in wl.lengths)
        point["length_as_host_int"] = figures(timed(int(uniform_len)))
    del ks, vs
    return point


def decode_curve(dev, iters=12):
    """The decode op over the range the target names: batch 64 at fixed context lengths 512 ... 4096
    (Qwen3-8B heads), the long-context configuration (cfg4), and the regime the engine runs in
    (batch 128, context lengths uniform in [128, 1280])."""
    from infer_amd import workloads
    points = []
    for ctx in (512, 1024, 2048, 4096):
        wl = workloads.make_decode_workload(f"b64-ctx{ctx}", [ctx] * 64, 32, 8, seed=ctx, q_scale=128 ** -0.5,
                                            device=dev, device_fill=True)
        pool_mb = 2 * wl.k_cache.numel() * 2 / 1e6
        points.append(decode_point(f"batch 64 x ctx {ctx}", wl, max(2, min(8, int(1100 / pool_mb) + 1)), iters,
                                   uniform_len=ctx))
        del wl
        torch.cuda.empty_cache()
    gen = torch.Generator().manual_seed(5)
    lens = torch.randint(128, 1281, (128,), generator=gen).tolist()
    wl = workloads.make_decode_workload("b128-engine", lens, 32, 8, seed=5, q_scale=128 ** -0.5, device=dev,
                                        device_fill=True)
    points.append(decode_point("batch 128 x ctx U[128,1280] (engine regime)", wl, 4, iters))
    del wl
    torch.cuda.empty_cache()
    wl = workloads.cfg4(device=dev, device_fill=True)
    points.append(decode_point("cfg4: batch 8 x ctx 32768, Hq=64", wl, 2, iters, uniform_len=32768))
    del wl
    torch.cuda.empty_cache()
    return points


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=200)
    ap.add_argument("--warmup", type=int, default=20)
    ap.add_argument("--copies", type=int, default=4, help="independent cache copies walked round-robin")
    ap.add_argument("--no-cpu", action="store_true", help="skip the CPU baseline legs")
    ap.add_argument("--no-curve", action="store_true", help="skip the decode curve of the default run")
    ap.add_argument("--splits", type=int, default=0, help="KV-split workgroups per decode call (0 = library default)")
    ap.add_argument("--counters", action="store_true",
                    help="short untimed run for `rocprofv3 --pmc`: a 1 GiB plain copy (x3), the decode op (x5), "
                         "a prefill-sized append (x3), the fused norm + RoPE + append (x3) and the prefill "
                         "attention (x3) of the same step")
    ap.add_argument("--decode-curve", action="store_true", help="only the decode curve, printed as JSON")
    ap.add_argument("--hybrid", action="store_true",
                    help="Merilorn beside Qwen3 at equal sizes: engine throughput and every kernel, printed as JSON")
    ap.add_argument("--vokelix", action="store_true",
                    help="Vokelix beside Qwen3 and Merilorn at equal sizes: engine throughput and every kernel, printed as JSON")
    ap.add_argument("--dogetar", action="store_true",
                    help="Dogetar beside Qwen3 and Vokelix at equal sizes: engine throughput and every kernel, printed as JSON")
    ap.add_argument("--tulurax", action="store_true",
                    help="Tulurax beside Qwen3 and Vokelix at equal sizes: engine throughput and every kernel, printed as JSON")
    ap.add_argument("--hybrid-kernels-only", action="store_true", help="with --hybrid, --vokelix, --dogetar or --tulurax: the kernels alone")
    ap.add_argument("--e2e", action="store_true",
                    help="end-to-end decode through the engine (random-init Qwen3, HIP-graph decode) instead "
                         "of the kernel benchmark")
    ap.add_argument("--e2e-model", default="8b", choices=["0.6b", "8b", "32b"])
    ap.add_argument("--e2e-batch", type=int, default=128)
    ap.add_argument("--e2e-new", type=int, default=256)
    ap.add_argument("--e2e-check", type=int, default=8,
                    help="decode steps at the start that run both eagerly and as graph replays and are compared")
    ap.add_argument("--no-e2e", action="store_true", help="skip the end-to-end leg of the default run")
    ap.add_argument("--e2e-eager", action="store_true", help="run the decode steps eagerly (no HIP graph)")
    args = ap.parse_args()
    if args.gpus != 1 or int(os.environ.get("WORLD_SIZE", "1")) != 1:
        print("bench.py measures one GPU: this path needs no collective and every box here has one GPU; "
              "run with --gpus 1", file=sys.stderr)
        sys.exit(2)
    if not torch.cuda.is_available():
        print("bench.py needs a GPU: the HIP kernels are the only implementation of the path", file=sys.stderr)
        sys.exit(2)

    if args.e2e:
        run_e2e(args)
        return
    for chosen, run in ((args.hybrid, run_hybrid), (args.vokelix, run_vokelix), (args.dogetar, run_dogetar), (args.tulurax, run_tulurax)):
        if chosen:
            run(args)
            return
    from infer_amd import ops, workloads
    dev = torch.device("cuda:0")
    if args.decode_curve:
        print(json.dumps({"decode_curve": decode_curve(dev)}))
        return

    p3_cpu = workloads.cfg3()                       # drawn on the CPU from the seed; also the CPU append baseline
    if args.counters:
        wl = workloads.cfg2(device=dev, device_fill=True)
        b, hq, hkv, d = len(wl.lengths), wl.num_q_heads, wl.num_kv_heads, wl.head_dim
        src = torch.empty(1 << 30, dtype=torch.uint8, device=dev).random_(0, 255)
        dst = torch.empty_like(src)
        out = torch.empty((b, hq, d), dtype=torch.bfloat16, device=dev)
        ws = ops.decode_workspace(dev, b, hq, hkv, d)
        p3 = p3_cpu.to(dev)
        torch.cuda.synchronize()
        for _ in range(3):
            dst.copy_(src)      # plain copy of known size: 1 GiB read, 1 GiB written
        for _ in range(5):
            ops.paged_attn_decode(wl.q, wl.k_cache, wl.v_cache, wl.block_table, wl.context_lens, wl.scale, out, ws)
        for _ in range(3):
            ops.store_kvcache(p3.k_new, p3.v_new, p3.k_cache, p3.v_cache, p3.slot_mapping)
        n_q = int(p3.q.shape[0])
        qkv = torch.randn((n_q, (hq + 2 * hkv) * d), dtype=torch.bfloat16, device=dev)
        q_, k_, v_ = (t.view(n_q, -1, d) for t in qkv.split([hq * d, hkv * d, hkv * d], dim=-1))
        w_ = torch.ones(d, dtype=torch.bfloat16, device=dev)
        cs_ = torch.randn((4096, d), dtype=torch.bfloat16, device=dev)
        pos_ = torch.randint(0, 4096, (n_q,), device=dev)
        sl_ = p3.slot_mapping[p3.row_of_query].contiguous()
        for _ in range(3):
            ops.qk_norm_rope_store_kvcache(q_, k_, v_, pos_, w_, w_, 1e-6, cs_, p3.k_cache, p3.v_cache, sl_,
                                           write_key=False)
        ops.store_kvcache(p3.k_new, p3.v_new, p3.k_cache, p3.v_cache, p3.slot_mapping)
        for _ in range(3):
            ops.flash_attn_varlen_func(p3.q, p3.k_cache, p3.v_cache, max_seqlen_q=p3.max_seqlen_q,
                                       cu_seqlens_q=p3.cu_seqlens_q, max_seqlen_k=p3.max_seqlen_k,
                                       cu_seqlens_k=p3.cu_seqlens_k, softmax_scale=p3.scale, causal=True,
                                       block_table=p3.block_table)
        # the decode op with the batch's length as one host integer (a single kernel, no merge): batch 64 x ctx 2048
        wu = workloads.make_decode_workload("b64-ctx2048", [2048] * 64, 32, 8, seed=2048, q_scale=128 ** -0.5,
                                            device=dev, device_fill=True)
        for _ in range(5):
            ops.paged_attn_decode(wu.q, wu.k_cache, wu.v_cache, wu.block_table, 2048, wu.scale, out, ws)
        torch.cuda.synchronize()
        pairs = sum((n - c) * c + (n - c) * (n - c + 1) // 2 for n, c in zip(p3.lengths, p3.cached))
        print(json.dumps({"counters_run": True, "copy_bytes": 1 << 30, "decode_algorithmic_bytes": wl.decode_bytes,
                          "uniform_decode_algorithmic_bytes": wu.decode_bytes,
                          "append_algorithmic_bytes": p3.append_bytes,
                          "fused_algorithmic_bytes": n_q * (2 * hq * d * 2 + 4 * hkv * d * 2),
                          "prefill_flops": 4 * p3.num_q_heads * p3.head_dim * pairs}))
        return

    wl = workloads.cfg2().to(dev)                   # the headline workload: seeded on the CPU, then moved
    b, hq, hkv, d = len(wl.lengths), wl.num_q_heads, wl.num_kv_heads, wl.head_dim
    k_copies = [wl.k_cache] + [torch.randn_like(wl.k_cache) for _ in range(args.copies - 1)]
    v_copies = [wl.v_cache] + [torch.randn_like(wl.v_cache) for _ in range(args.copies - 1)]
    out = torch.empty((b, hq, d), dtype=torch.bfloat16, device=dev)
    ws = ops.decode_workspace(dev, b, hq, hkv, d)
    it = [0]

    def step():
        i = it[0] % args.copies
        it[0] += 1
        ops.paged_attn_decode(wl.q, k_copies[i], v_copies[i], wl.block_table, wl.context_lens, wl.scale, out, ws,
                              split_workgroups=args.splits)

    def split_only():
        i = it[0] % args.copies
        it[0] += 1
        ops.paged_attn_decode_split(wl.q, k_copies[i], v_copies[i], wl.block_table, wl.context_lens, wl.scale, ws,
                                    split_workgroups=args.splits)

    # An idle GPU needs tens of milliseconds of work to reach its steady clocks; a short run (say 5 warm-up
    # and 20 timed steps = 3 ms) would otherwise time the ramp.  The op is therefore repeated, untimed,
    # for `spin_up_s` before the W warm-up steps and the exactly K timed steps.
    spin_up_s = 0.25
    t_spin = time.perf_counter()
    while time.perf_counter() - t_spin < spin_up_s:
        for _ in range(50):
            step()
        torch.cuda.synchronize()
    # whole op, exactly K steps
    for _ in range(args.warmup):
        step()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(args.steps):
        step()
    torch.cuda.synchronize()
    wall_ms = (time.perf_counter() - t0) * 1e3 / args.steps
    ms_per_step = gpu_time_ms(step, args.steps, 0)
    ms_per_step = max(ms_per_step, 1e-6)
    nbytes = wl.decode_bytes
    value = nbytes / (ms_per_step * 1e-3) / 1e9

    # dominant kernel alone (the KV-streaming split kernel)
    split_ms = gpu_time_ms(split_only, args.steps, 5)
    achieved = nbytes / (split_ms * 1e-3) / 1e9

    # KV append: decode-sized (64 rows, latency bound) and prefill-sized (cfg3)
    ap_small_ms = gpu_time_ms(lambda: ops.store_kvcache(wl.k_new, wl.v_new, wl.k_cache, wl.v_cache, wl.slot_mapping),
                              args.steps, 5)
    p3 = p3_cpu.to(dev)
    reps = 24   # distinct source/destination buffers walked round-robin (24 x ~100 MB > Infinity Cache)
    srcs = [(torch.randn_like(p3.k_new), torch.randn_like(p3.v_new)) for _ in range(reps)]
    dsts = [(torch.empty_like(p3.k_cache), torch.empty_like(p3.v_cache)) for _ in range(reps)]
    jt = [0]

    def append_step():
        j = jt[0] % reps
        jt[0] += 1
        ops.store_kvcache(srcs[j][0], srcs[j][1], dsts[j][0], dsts[j][1], p3.slot_mapping)

    ap_ms = gpu_time_ms_median(append_step, max(args.steps, 48), reps)
    append_gbs = p3.append_bytes / (ap_ms * 1e-3) / 1e9
    # fused QK-norm + RoPE + append (one launch for the four steps in front of attention), over rotated
    # qkv buffers and cache pairs (> 512 MB in total) so that every launch reads and writes HBM
    def fused_case(n_rows):
        d_ = 128
        row = (hq + 2 * hkv) * d_
        nbuf = max(2, min(reps, (700 << 20) // (n_rows * row * 2) + 1))
        qkvs = [torch.randn((n_rows, row), dtype=torch.bfloat16, device=dev) for _ in range(nbuf)]
        w_ = torch.ones(d_, dtype=torch.bfloat16, device=dev)
        cs_ = torch.randn((4096, d_), dtype=torch.bfloat16, device=dev)
        pos_ = torch.randint(0, 4096, (n_rows,), device=dev)
        sl_ = torch.randperm(p3.k_cache.shape[0] * 256, device=dev)[:n_rows].to(torch.int32)
        ft = [0]

        def fused_step():
            j = ft[0]
            ft[0] += 1
            q_, k_, v_ = (t.view(n_rows, -1, d_) for t in qkvs[j % nbuf].split([hq * d_, hkv * d_, hkv * d_], dim=-1))
            kc_, vc_ = dsts[j % reps]
            ops.qk_norm_rope_store_kvcache(q_, k_, v_, pos_, w_, w_, 1e-6, cs_, kc_, vc_, sl_, write_key=False)
        ms_ = gpu_time_ms_median(fused_step, 48, 6)
        nbytes_ = n_rows * (2 * hq * d_ * 2 + 4 * hkv * d_ * 2)   # q read + written in place, k and v read, both stored
        return round(ms_ * 1e3, 2), round(nbytes_ / ms_ / 1e6, 1), nbuf
    fused_small = fused_case(b)
    fused_big = fused_case(int(p3.q.shape[0]))

    # paged varlen causal prefill attention on the same cfg3 step (after its append), for the record
    kc3, vc3 = p3.k_cache.clone(), p3.v_cache.clone()
    ops.store_kvcache(p3.k_new, p3.v_new, kc3, vc3, p3.slot_mapping)
    def prefill_step():
        ops.flash_attn_varlen_func(
            p3.q, kc3, vc3, max_seqlen_q=p3.max_seqlen_q, cu_seqlens_q=p3.cu_seqlens_q, max_seqlen_k=p3.max_seqlen_k,
            cu_seqlens_k=p3.cu_seqlens_k, softmax_scale=p3.scale, causal=True, block_table=p3.block_table)
    pf_ms = gpu_time_ms_median(prefill_step, 40, 10)
    pairs = sum((n - c) * c + (n - c) * (n - c + 1) // 2 for n, c in zip(p3.lengths, p3.cached))
    pf_flops = 4 * p3.num_q_heads * p3.head_dim * pairs

    # the front end and the prefill attention back to back, the attention reading the query rows the front
    # end has just written (the order of a prefill step in the engine): what the choice of cache hints
    # in the front end is judged by
    n3 = int(p3.q.shape[0])
    qkv3 = [torch.randn((n3, (hq + 2 * hkv) * d), dtype=torch.bfloat16, device=dev) for _ in range(6)]
    w3 = torch.ones(d, dtype=torch.bfloat16, device=dev)
    cs3 = torch.randn((4096, d), dtype=torch.bfloat16, device=dev)
    pos3 = torch.randint(0, 4096, (n3,), device=dev)
    sl3 = p3.slot_mapping[p3.row_of_query].contiguous()
    pt = [0]

    def front_then_attention():
        j = pt[0]
        pt[0] += 1
        q_, k_, v_ = (t.view(n3, -1, d) for t in qkv3[j % 6].split([hq * d, hkv * d, hkv * d], dim=-1))
        ops.qk_norm_rope_store_kvcache(q_, k_, v_, pos3, w3, w3, 1e-6, cs3, kc3, vc3, sl3, write_key=False)
        ops.flash_attn_varlen_func(q_, kc3, vc3, max_seqlen_q=p3.max_seqlen_q, cu_seqlens_q=p3.cu_seqlens_q,
                                   max_seqlen_k=p3.max_seqlen_k, cu_seqlens_k=p3.cu_seqlens_k, softmax_scale=p3.scale,
                                   causal=True, block_table=p3.block_table)
    pair_ms = gpu_time_ms_median(front_then_attention, 24, 6)
    del qkv3

    line = {
        "metric": "paged decode attn HBM GB/s (% of 8 TB/s peak), Qwen3-8B shapes bs=64",
        "value": round(value, 1), "unit": "GB/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(ms_per_step, 5), "higher_is_better": True, "scaling": "weak",
        "vs_baseline": None, "dtype": "bf16", "data": "synthetic",
        "config": {"workload": "cfg2: paged decode attention, Hq=32 Hkv=8 D=128 block=256 batch=64 "
                               "ctx~U[512,4096] (seed 0), tables shuffled over a 1.2x pool",
                   "tokens": sum(wl.lengths), "algorithmic_bytes": nbytes, "cache_copies": args.copies,
                   "split_workgroups": args.splits or "default"},
        "pct_of_peak": round(100.0 * value / HBM_PEAK_GBS, 2),
        "spin_up_s": spin_up_s,
        "wall_ms_per_step": round(wall_ms, 5),
        "roofline": {"bound": "hbm", "kernel": "paged_decode_kernel<true>", "achieved": round(achieved, 1),
                     "peak": HBM_PEAK_GBS, "unit": "GB/s", "frac": round(achieved / HBM_PEAK_GBS, 4),
                     "traffic": MEASURED_TRAFFIC_BYTES, "traffic_source": TRAFFIC_SOURCE,
                     "avg_kernel_ms": round(split_ms, 5)},
        "append": {"decode_rows": b, "decode_us": round(ap_small_ms * 1e3, 2),
                   "prefill_rows": int(p3.slot_mapping.numel()), "prefill_bytes": p3.append_bytes,
                   "prefill_us": round(ap_ms * 1e3, 2), "prefill_GBps": round(append_gbs, 1),
                   "prefill_frac_of_peak": round(append_gbs / HBM_PEAK_GBS, 4)},
    }
    line["prefill_attention"] = {"workload": "cfg3: 16 prompts U[64,2048], 0-50 % cached, causal over the paged cache",
                                 "query_tokens": int(p3.q.shape[0]), "ms": round(pf_ms, 4),
                                 "TFLOPs": round(pf_flops / (pf_ms * 1e-3) / 1e12, 1),
                                 "frac_of_bf16_mfma_peak": round(pf_flops / (pf_ms * 1e-3) / 1e12 / 2500.0, 4)}
    line["fused_qk_norm_rope_append"] = {"decode_rows": b, "decode_us": fused_small[0],
                                         "prefill_rows": int(p3.q.shape[0]), "prefill_us": fused_big[0],
                                         "prefill_GBps": fused_big[1],
                                         "prefill_frac_of_peak": round(fused_big[1] / HBM_PEAK_GBS, 4),
                                         "front_end_then_prefill_attention_us": round(pair_ms * 1e3, 2),
                                         "note": f"{fused_big[2]} qkv buffers and {reps} cache pairs walked round-robin "
                                                 "(> 512 MB): an HBM figure; bytes = q in + q out + k in + v in + "
                                                 "k and v stored"}
    del k_copies, v_copies, srcs, dsts, kc3, vc3
    torch.cuda.empty_cache()
    if not args.no_curve:
        line["decode_curve"] = decode_curve(dev)
    if not args.no_cpu:
        line["cpu_baseline"] = cpu_baseline()
        line["cpu_baselines_other_configs"] = cpu_baselines_other(p3_cpu)
    if not args.no_e2e:
        # the end-to-end configuration runs in a child process of its own (it sizes its KV pool from the
        # free HBM); its JSON line is attached as a secondary figure and never affects `value`
        del wl, p3, out, ws
        torch.cuda.empty_cache()
        import subprocess
        try:
            child = subprocess.run([sys.executable, os.path.abspath(__file__), "--e2e"], capture_output=True,
                                   text=True, timeout=600)
            line["e2e_decode"] = json.loads(child.stdout.strip().splitlines()[-1])
        except Exception as exc:  # noqa: BLE001
            line["e2e_decode"] = {"error": f"{type(exc).__name__}: {exc}"[:200]}
    print(json.dumps(line))


if __name__ == "__main__":
    main()
