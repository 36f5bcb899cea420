"""Merilorn without a GPU: the oracle against other ways to compute the same, configuration and loading, the
portion scheduler, the step plan."""
import json

import numpy as np
import pytest
import torch

from infer_amd.block_manager import BlockManager, SlotPool
from infer_amd.config import Config, MerilornConfig, ModelConfig, load_model_config
from infer_amd.layers import PackedLinear, yarn_rotary_table
from infer_amd.merilorn import MerilornForCausalLM
from infer_amd.registry import model_class
from infer_amd.sampling_params import SamplingParams
from infer_amd.scheduler import PortionScheduler
from infer_amd.sequence import Sequence, SequenceStatus
from infer_amd.step_plan import CHUNK, DENSE_FROM, build
from infer_amd.weight_loader import load_model
from oracle import merilorn_ref as ref
from tests import merilorn_helpers as mh


# ------------------------------------------------------------------ the oracle
def test_rotation_depends_on_distance_only_and_leaves_the_rest_alone():
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((2, 12))
    freq, mag = ref.yarn_frequencies(8, 100.0)
    assert mag == 1.0
    for a, b in ((3, 1), (40, 38)):
        x = ref.rotate_interleaved(np.stack([q, k]), [a, b], freq)
        assert np.isclose(x[0] @ x[1], ref.rotate_interleaved(np.stack([q, k]), [2, 0], freq)[0] @ k)
        assert np.array_equal(x[:, 8:], np.stack([q, k])[:, 8:])
    one = ref.rotate_interleaved(np.array([[1.0, 0.0, 0.0, 2.0]]), [1], np.array([0.5, 0.25]))
    assert np.allclose(one, [[np.cos(.5), np.sin(.5), -2 * np.sin(.25), 2 * np.cos(.25)]])


@pytest.mark.parametrize("scaling", [None, mh.ROT["scaling"], dict(factor=8.0, original=64, fast=1.0, slow=1.0),
                                     dict(factor=3.0, original=4096, fast=1e9, slow=1e-9)])
def test_rotary_table_is_the_oracles(scaling):
    dims, base = 24, 5000.0
    table = yarn_rotary_table(dims, 300, base, scaling, "cpu").numpy()
    freq, mag = ref.yarn_frequencies(dims, base, scaling)
    angle = np.arange(300)[:, None] * freq
    assert np.allclose(table[..., 0], np.cos(angle) * mag, atol=1e-6) and np.allclose(table[..., 1], np.sin(angle) * mag, atol=1e-6)
    if scaling and scaling["fast"] > 1e6:            # a ramp over all pairs: the first is kept, the last is slowed down
        assert freq[0] == 1.0 and freq[-1] < base ** (-22 / 24)


def test_delta_scan_equals_its_chunk_form():
    """The algebra of the chunked kernels, in numpy: U = T (beta V) - T (beta e^G K) S."""
    rng = np.random.default_rng(1)
    n, dim, vdim = 13, 6, 5
    q, k = ref.unit_norm(rng.standard_normal((2, n, dim)))
    v, beta = rng.standard_normal((n, vdim)), ref.sigmoid(rng.standard_normal(n))
    g = -np.abs(rng.standard_normal((n, dim))) * 3
    s0 = rng.standard_normal((dim, vdim))
    want, s_want = ref.delta_scan(q, k, v, g, beta, s0)
    G = np.cumsum(g, 0)
    e = np.exp(np.minimum(G[:, None] - G[None], 0))
    A = np.einsum("id,jd,ijd->ij", k, k, e)
    B = np.einsum("id,jd,ijd->ij", q, k, e)
    T = np.linalg.inv(np.eye(n) + np.tril(beta[:, None] * A, -1)) * beta
    U = T @ v - T @ (k * np.exp(G)) @ s0
    assert np.allclose((q * np.exp(G)) @ s0 + np.tril(B) @ U, want)
    assert np.allclose(np.exp(G[-1])[:, None] * s0 + (k * np.exp(G[-1] - G)).T @ U, s_want)
    half, s_half = ref.delta_scan(q[:7], k[:7], v[:7], g[:7], beta[:7], s0)
    rest, s_rest = ref.delta_scan(q[7:], k[7:], v[7:], g[7:], beta[7:], s_half)
    assert np.allclose(np.concatenate([half, rest]), want) and np.allclose(s_rest, s_want)


def test_causal_conv_looks_back_and_never_ahead():
    x, taps = np.zeros((6, 2)), np.array([[1.0, 2.0, 3.0], [4.0, 5.0, 6.0]])
    x[2] = 1.0
    assert np.array_equal(ref.causal_conv(x, taps)[:, 0], [0, 0, 3, 2, 1, 0])
    assert np.array_equal(ref.causal_conv(x, taps)[:, 1], [0, 0, 6, 5, 4, 0])


def test_attention_over_latents_equals_attention_over_keys():
    """Scores and values by way of the latent space (W_uk^T q, W_uv sum) are the same numbers."""
    m, rng = mh.latent()["mixer"], np.random.default_rng(2)
    h = rng.standard_normal((9, 20))
    shapes = {"q": (3 * 24, 20), "dkv": (48, 20), "dkv.norm": (40,), "uk": (48, 40), "uv": (72, 40), "g": (3, 20), "o": (20, 72)}
    w = {k: rng.standard_normal(s) * 0.3 for k, s in shapes.items()}
    want = ref.latent_attention(h, m, w.get, 1e-5)
    freq, mag = ref.yarn_frequencies(8, ROT_BASE, mh.ROT["scaling"])
    q = (h @ w["q"].T).reshape(9, 3, 24)
    down = h @ w["dkv"].T
    c = ref.rms_norm(down[:, :40], w["dkv.norm"], 1e-5)
    row = np.concatenate([c, ref.rotate_interleaved(down[:, 40:], np.arange(9), freq, mag)], -1)
    qx = np.concatenate([np.einsum("thd,hdr->thr", q[..., :16], w["uk"].reshape(3, 16, 40)),
                         ref.rotate_interleaved(q[..., 16:], np.arange(9), freq, mag)], -1)
    o = np.zeros((9, 3, 24))
    for t in range(9):
        s = qx[t] @ row[:t + 1].T * m["scale"]
        p = np.exp(s - s.max(-1, keepdims=True))
        o[t] = np.einsum("hr,hvr->hv", p / p.sum(-1, keepdims=True) @ c[:t + 1], w["uv"].reshape(3, 24, 40))
    o = o * ref.sigmoid(h @ w["g"].T)[..., None]
    assert np.allclose(o.reshape(9, 72) @ w["o"].T, want)


ROT_BASE = mh.ROT["base"]


# ------------------------------------------------------------------ configuration and weights
def test_config_and_registry(tmp_path):
    config = mh.small_config()
    folder = mh.save_model(tmp_path / "m", config, mh.make_weights(config))
    cfg = load_model_config(folder)
    assert isinstance(cfg, MerilornConfig) and model_class(cfg) is MerilornForCausalLM
    assert [s.owner for s in cfg.layers] == [0, 1, 2, 1, 4, 0, 2]
    assert [s.ff for s in cfg.layers] == [None, 56, 48, 56, None, None, 48]
    assert (cfg.layers[0].mixer["decay_rank"], cfg.layers[6].mixer["gate_rank"]) == (12, 20)
    assert Config(folder, kvcache_block_size=64, dtype="float32").hf_config.torch_dtype == torch.float32
    with pytest.raises(ValueError, match="does not run"):
        Config(hf_config=ModelConfig(), dtype="float32")
    (tmp_path / "other").mkdir()
    (tmp_path / "other" / "config.json").write_text(json.dumps({"architecture": "Nobody"}))
    with pytest.raises(ValueError, match="Nobody"):
        load_model_config(str(tmp_path / "other"))
    (tmp_path / "q").mkdir()
    (tmp_path / "q" / "config.json").write_text(json.dumps({"architectures": ["Qwen3ForCausalLM"], "hidden_size": 64, "num_attention_heads": 2}))
    assert isinstance(load_model_config(str(tmp_path / "q")), ModelConfig)


def test_every_tensor_lands_in_its_place(tmp_path):
    config = mh.small_config()
    weights = mh.make_weights(config)
    folder = mh.save_model(tmp_path / "m", config, weights)
    cfg = load_model_config(folder)
    model = MerilornForCausalLM.build(cfg, "cpu")
    assert load_model(model, folder) == len(weights)
    block = model.blocks["0"].mixer
    assert np.array_equal(block.in_proj.piece(block.in_proj.weight.data.T, "k").T.double().numpy(), weights["l0.mix.k"])
    assert np.array_equal(block.in_proj.piece(block.in_proj.weight.data.T, "g1").T.double().numpy(), weights["l0.mix.g1"])
    qk = 2 * 24
    assert np.array_equal(block.conv.weight.double().numpy()[qk:2 * qk], weights["l0.mix.k.conv"])
    assert block.conv.weight.dtype == torch.float32 and block.in_proj.weight.dtype == torch.bfloat16
    for shape, bad in (((3, 3), ValueError), (None, KeyError)):
        w = dict(weights)
        if shape is None:
            del w["l1.mix.g"]
        else:
            w["l1.mix.g"] = np.zeros(shape)
        broken = mh.save_model(tmp_path / f"bad{bad.__name__}", config, w)
        with pytest.raises(bad):
            load_model(MerilornForCausalLM.build(cfg, "cpu"), broken)
    w = dict(weights)
    w["l3.norm1"] = np.zeros(72)                      # a layer that uses another's weights has none of its own
    with pytest.raises(KeyError, match="l3"):
        load_model(MerilornForCausalLM.build(cfg, "cpu"), mh.save_model(tmp_path / "extra", config, w))


def test_packed_linear_pieces_start_aligned():
    lin = PackedLinear(4, {"q": 6, "k": 3, "v": 5, "b": 2}, torch.float32, dense=("q",))
    assert lin.offset == {"q": 0, "k": 6, "v": 16, "b": 24} and lin.weight.shape == (64, 4)
    lin.weight_loader(lin.weight, torch.ones(5, 4), "v")
    assert float(lin.weight.sum()) == 20
    with pytest.raises(ValueError):
        lin.weight_loader(lin.weight, torch.ones(4, 4), "v")


# ------------------------------------------------------------------ scheduler and pools
def test_reserve_takes_all_or_nothing_and_returns_blocks():
    pool = BlockManager(4, 64)
    seq = Sequence([1] * 100, block_size=64)
    assert seq.num_blocks == 2 and Sequence([1] * 100).num_blocks == 1
    assert pool.reserve(seq, 65) and len(seq.block_table) == 2 and pool.reserve(seq, 128) and len(seq.block_table) == 2
    other = Sequence([2], block_size=64)
    assert not pool.reserve(other, 129) and other.block_table == [] and pool.num_free_blocks == 2
    assert pool.reserve(other, 128) and pool.num_free_blocks == 0 and set(seq.block_table).isdisjoint(other.block_table)
    pool.deallocate(seq)
    assert pool.num_free_blocks == 2 and seq.block_table == []


def test_slot_pool():
    pool = SlotPool(2)
    assert [pool.take(), pool.take()] == [0, 1]
    with pytest.raises(RuntimeError):
        pool.take()
    pool.give_back(0)
    with pytest.raises(RuntimeError):
        pool.give_back(0)
    assert pool.take() == 0


def _engine_config(**kw):
    cfg = MerilornConfig(16, 8)
    base = dict(hf_config=cfg, kvcache_block_size=32, num_kvcache_blocks=8, max_num_seqs=3, max_model_len=256, max_num_batched_tokens=256)
    return Config(**{**base, **kw})


def _run(sched, steps=200):
    """Drives the scheduler with token 7; returns the portions of every step as (id, count)."""
    log = []
    while not sched.is_finished():
        portions = sched.schedule()
        held = [s.state_slot for s in sched.running]
        assert len(set(held)) == len(held) and min(held) >= 0
        blocks = [b for s in sched.running for b in s.block_table]
        assert len(set(blocks)) == len(blocks)
        for p in portions:
            assert p.count >= 1 and len(p.seq.block_table) * 32 >= p.seq.num_computed_tokens + p.count
        log.append([(p.seq.seq_id, p.count) for p in portions])
        sched.postprocess(portions, [7] * sum(p.last for p in portions))
        assert len(log) < steps
    return log


def test_portions_decoded_tokens_first_then_prompts_within_the_budget():
    sched = PortionScheduler(_engine_config(max_model_len=100, max_num_batched_tokens=100))
    a, b = Sequence([1] * 30, SamplingParams(0, 4, True), 32), Sequence([2] * 90, SamplingParams(0, 2, True), 32)
    sched.add(a)
    sched.add(b)
    log = _run(sched)
    assert log == [[(a.seq_id, 30), (b.seq_id, 70)], [(a.seq_id, 1), (b.seq_id, 20)], [(a.seq_id, 1), (b.seq_id, 1)], [(a.seq_id, 1)]]
    assert a.completion_token_ids == [7] * 4 and sched.block_manager.num_free_blocks == 8 and sched.slots.num_free == 3


def test_state_slots_limit_how_many_run():
    sched = PortionScheduler(_engine_config(max_num_seqs=2))
    seqs = [Sequence([i] * 5, SamplingParams(0, 3, True), 32) for i in range(1, 6)]
    for s in seqs:
        sched.add(s)
    log = _run(sched)
    assert max(map(len, log)) == 2 and all(s.completion_token_ids == [7] * 3 for s in seqs)


def test_preempted_sequence_starts_over_from_its_first_token():
    sched = PortionScheduler(_engine_config(num_kvcache_blocks=4))
    a, b = Sequence([1] * 60, SamplingParams(0, 10, True), 32), Sequence([2] * 60, SamplingParams(0, 10, True), 32)
    sched.add(a)
    sched.add(b)
    log = _run(sched)
    flat = [x for step in log for x in step]
    assert (b.seq_id, 60) in flat and any(i == b.seq_id and n > 60 for i, n in flat)      # with what it had generated
    assert len(a.completion_token_ids) == len(b.completion_token_ids) == 10
    assert sched.block_manager.num_free_blocks == 4 and sched.slots.num_free == 3


def test_what_can_never_run_is_refused():
    sched = PortionScheduler(_engine_config(num_kvcache_blocks=2))
    with pytest.raises(ValueError):
        sched.add(Sequence([1] * 257, SamplingParams(0, 1, True), 32))
    sched.add(Sequence([1] * 65, SamplingParams(0, 1, True), 32))
    with pytest.raises(AssertionError):
        sched.schedule()
    ended = PortionScheduler(_engine_config(max_model_len=32))
    s = Sequence([1] * 30, SamplingParams(0, 50, True), 32)
    ended.add(s)
    _run(ended)
    assert s.status is SequenceStatus.FINISHED and len(s) == 33       # the token behind the last one that fits


# ------------------------------------------------------------------ step plan
def test_step_plan_against_a_plain_loop():
    rng = np.random.default_rng(3)
    bs, portions = 32, []
    blocks = list(rng.permutation(60))
    for slot, (lo, n) in enumerate([(40, 1), (0, 70), (17, 2), (0, 1), (33, 33), (64, 64), (5, 16)]):
        seq = Sequence([int(t) for t in rng.integers(0, 99, lo + n + 3)], block_size=bs)
        seq.num_computed_tokens, seq.state_slot = lo, slot
        seq.block_table = [int(blocks.pop()) for _ in range(-(-(lo + n) // bs))]
        portions.append((seq, n))
    plan, first = build(portions, bs, 4, 7, 60, "cpu")
    order = sorted(range(7), key=lambda i: portions[i][1])
    assert plan.decode_rows == 2 and plan.rows == sum(n for _, n in portions)
    seen = 0
    for s, i in enumerate(order):
        seq, n = portions[i]
        lo = seq.num_computed_tokens
        assert first[i] == seen
        for t in range(n):
            r, p = seen + t, lo + t
            assert int(plan.input_ids[r]) == seq.token_ids[p] and int(plan.positions[r]) == p and int(plan.row_ctx[r]) == p + 1
            assert int(plan.slot_mapping[r]) == seq.block_table[p // bs] * bs + p % bs and int(plan.row_seq[r]) == s
            assert plan.ring_slot[r].tolist() == [seq.state_slot, n - 1 - t]
        assert plan.block_tables[s, :len(seq.block_table)].tolist() == seq.block_table
        seen += n
    assert plan.state_slots.tolist() == [0, 3]
    covered = []
    for c0, nc, slot, lo in plan.portions.tolist():
        seq, n = portions[slot]
        assert lo == seq.num_computed_tokens and nc == -(-n // CHUNK)
        for r0, cnt, p0, start, sl, _ in plan.chunks[c0:c0 + nc].tolist():
            assert start == lo and sl == slot and p0 - lo == r0 - first[slot]
            covered += range(r0, r0 + cnt)
    assert covered == list(range(2, plan.rows))
    dense = [i for i in order if portions[i][1] >= DENSE_FROM]
    assert plan.dense_row == first[dense[0]] and plan.dense_cu_q.tolist() == [0, 64, 134] and plan.dense_cu_k.tolist() == [0, 128, 198]
    assert (plan.dense_keys, plan.dense_max_q, plan.dense_max_k) == (198, 70, 128)
    with pytest.raises(RuntimeError):
        build([(portions[0][0], 80)], bs, 4, 7, 60, "cpu")
    with pytest.raises(RuntimeError):
        build([(portions[4][0], 33)], bs, 4, 4, 60, "cpu")           # slot 4 of 4
