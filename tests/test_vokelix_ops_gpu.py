"""The kernels of grouped attention, of linear attention with a constant decay and of the post-norm residual stream,
each alone, against ``oracle/vokelix_ref.py`` (float64) on random inputs made so that a wrong key, token or state shows."""
import numpy as np
import pytest
import torch

from infer_amd import hybrid_ops as ho, ops
from infer_amd.layers import yarn_rotary_table
from oracle import vokelix_ref as ref
from oracle.merilorn_ref import rms_norm, sigmoid, silu
from tests.test_hybrid_ops_gpu import BOTH, close, dev, host, rounded, tol

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------ residual stream
@BOTH
@pytest.mark.parametrize("width", [8, 72, 129, 1000, 2563, 4096])
def test_post_norm_forms(gpu, dtype, width):
    rng = np.random.default_rng(width)
    n, eps, alpha = 5, 1e-2, 1.9
    x0, y = rng.standard_normal((n, width)), rounded(rng.standard_normal((n, width)) * .3, dtype)
    wp, wn = 1 + rng.standard_normal((2, width)) * .3
    embed = rounded(rng.standard_normal((11, width)), dtype)
    want = rms_norm(alpha * x0 + y, wp, eps)
    for last in (None, dev(wn)):
        x = dev(x0)
        h = ho.post_norm(x, eps, y=dev(y, dtype), w_post=dev(wp), alpha=alpha, w_last=last, dtype=dtype)
        close(x, want, 2e-6)
        close(h, want if last is None else rms_norm(want, wn, eps), tol(dtype, 2e-6, 8e-3))
    x = torch.full((n, width), float("nan"), device="cuda")
    ids = torch.tensor([3, 0, 10, 10, 7], device="cuda")
    h = ho.post_norm(x, eps, tokens=ids, embed=dev(embed, dtype), dtype=dtype)
    assert np.array_equal(host(x), embed[ids.cpu()]) and np.array_equal(host(h), embed[ids.cpu()])


def test_post_norm_of_split_k_pieces(gpu):
    rng = np.random.default_rng(0)
    m, n, k = 7, 512, 4096
    a, w = dev(rng.standard_normal((m, k)), torch.bfloat16), dev(rng.standard_normal((n, k)) * .02, torch.bfloat16)
    y = ops.linear(a, w, defer=True)
    assert isinstance(y, ops.SplitKSum)
    x, wp = dev(rng.standard_normal((m, n))), 1 + rng.standard_normal(n) * .2
    want = rms_norm(2.5 * host(x) + host(a) @ host(w).T, wp, 1e-6)
    ho.post_norm(x, 1e-6, y=y, w_post=dev(wp), alpha=2.5, dtype=torch.bfloat16)
    close(x, want, 1e-5)


@BOTH
@pytest.mark.parametrize("d", [8, 30, 352])
def test_silu_and_mul(gpu, dtype, d):
    x = rounded(np.random.default_rng(d).standard_normal((6, 2 * d)) * 4, dtype)
    x[0, 0], x[1, 0] = 60.0, -60.0
    close(ho.silu_and_mul(dev(x, dtype)), silu(x[:, :d]) * x[:, d:], tol(dtype, 1e-6, 4e-3))


# ------------------------------------------------------------------ grouped attention
def up32(n):
    return -(-n // 32) * 32


@BOTH
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot", [(6, 2, 24, 16, 16), (4, 4, 32, 64, 32), (3, 1, 10, 7, 4), (5, 5, 9, 8, 6),
                                                         (16, 2, 128, 128, 64), (64, 8, 128, 96, 128), (8, 1, 64, 32, 0)])
@pytest.mark.parametrize("own", [True, False], ids=["keys", "queries-only"])
def test_grouped_front(gpu, dtype, heads, kv_heads, dim, vdim, rot, own):
    rng = np.random.default_rng(heads * dim)
    n, bs, nblk, eps, qx_rows = 7, 32, 3, 1e-2, 3
    koff = -(-heads * dim // 8) * 8
    voff = koff + -(-kv_heads * dim // 8) * 8
    cols = voff + kv_heads * vdim + 5
    cols += -cols % 8
    x = rounded(rng.standard_normal((n, cols)), dtype)
    bias, qn, kn = rng.standard_normal(cols), 1 + .3 * rng.standard_normal(heads * dim), 1 + .3 * rng.standard_normal(kv_heads * dim)
    pos, slots = rng.integers(0, 200, n), np.array([5, 31, 32, -1, 64, 95, 200], np.int32)      # one padding row, one outside the pool
    scaling = dict(factor=3.0, original=64, fast=8.0, slow=1.0)
    table = yarn_rotary_table(rot, 256, 777.0, scaling if rot else None, gpu)
    dp, vp = up32(dim), up32(vdim)
    cache = torch.full((nblk, kv_heads, bs, vp + dp), 7.0, dtype=dtype, device=gpu)
    qx = torch.full((qx_rows, heads, dp), float("nan"), dtype=dtype, device=gpu)
    proj = dev(x, dtype)
    ho.grouped_front(proj, heads, kv_heads if own else 0, dim, vdim, koff, voff, dev(bias), dev(qn), dev(kn), eps, table, rot,
                     dev(pos, torch.int64), dev(slots, torch.int32), cache, dp, vp, qx, qx_rows)
    freq, mag = ref.yarn_frequencies(rot, 777.0, scaling) if rot else (np.zeros(0), 1.0)

    def turned(cols, w, h):
        return ref.rotate_interleaved(rms_norm(cols, w, eps).reshape(n, h, dim), pos, freq, mag)

    q = turned(x[:, :heads * dim] + bias[:heads * dim], qn, heads)
    k = turned((x + bias)[:, koff:koff + kv_heads * dim], kn, kv_heads)
    v = (x + bias)[:, voff:voff + kv_heads * vdim].reshape(n, kv_heads, vdim)
    t = tol(dtype, 2e-6, 8e-3)
    close(qx[:, :, :dim], q[:qx_rows], t)
    assert not qx[:, :, dim:].any()
    close(proj[qx_rows:, :heads * dim], q[qx_rows:].reshape(n - qx_rows, -1), t)
    assert np.array_equal(host(proj[:qx_rows]), x[:qx_rows]) and np.array_equal(host(proj[:, heads * dim:]), x[:, heads * dim:])
    got = host(cache).transpose(0, 2, 1, 3).reshape(nblk * bs, kv_heads, vp + dp)
    for i, slot in enumerate(slots):
        if own and 0 <= slot < nblk * bs:
            close(torch.tensor(got[slot, :, vp:vp + dim]), k[i], t)
            close(torch.tensor(got[slot, :, :vdim]), v[i], t)
            assert not got[slot, :, vdim:vp].any() and not got[slot, :, vp + dim:].any()
    untouched = [s for s in range(nblk * bs) if not own or s not in slots]
    assert (got[untouched] == 7.0).all()


class Pages:
    """Random keys and values of several sequences in shuffled pages; every row that belongs to nobody is NaN."""

    def __init__(self, rng, lens, kv_heads, dim, vdim, bs, dtype):
        self.dim, self.vdim, self.dp, self.vp = dim, vdim, up32(dim), up32(vdim)
        self.k = [rounded(rng.standard_normal((n, kv_heads, dim)), dtype) for n in lens]
        self.v = [rounded(rng.standard_normal((n, kv_heads, vdim)), dtype) for n in lens]
        counts = [-(-n // bs) for n in lens]
        self.tables = np.full((len(lens), max(counts) + 1), -1, np.int32)
        ids = rng.permutation(sum(counts) + 2)
        self.cache = np.full((sum(counts) + 2, kv_heads, bs, self.vp + self.dp), np.nan)
        at = 0
        for s, n in enumerate(lens):
            for b in range(counts[s]):
                block = self.tables[s, b] = ids[at]
                at += 1
                m = min(bs, n - b * bs)
                rows = self.cache[block, :, :m]
                rows[:] = 0.0
                rows[..., :vdim] = self.v[s][b * bs:b * bs + m].transpose(1, 0, 2)
                rows[..., self.vp:self.vp + dim] = self.k[s][b * bs:b * bs + m].transpose(1, 0, 2)

    def queries(self, q, dtype):
        qx = np.zeros((*q.shape[:2], self.dp))
        qx[..., :self.dim] = q
        return dev(qx, dtype)


def one_query(q, k, v, scale, sink):
    """``q`` [heads, dim] sees all of ``k`` [keys, kv_heads, dim]."""
    group = len(q) // k.shape[1]
    s = np.einsum("hd,khd->hk", q, np.repeat(k, group, 1)) * scale
    top = np.maximum(s.max(-1), sink)[:, None]
    p = np.exp(s - top)
    return np.einsum("hk,khd->hd", p, np.repeat(v, group, 1)) / (p.sum(-1) + np.exp(sink - top[:, 0]))[:, None]


SHAPES = [(6, 2, 24, 16), (4, 1, 64, 64), (1, 1, 10, 7), (8, 8, 128, 128), (32, 4, 128, 128), (40, 2, 96, 32), (2, 1, 256, 200),
          (20, 1, 16, 48), (4, 2, 320, 300)]


@BOTH
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", SHAPES)
@pytest.mark.parametrize("splits", [0, 1, 5])
def test_grouped_attention_rows(gpu, dtype, heads, kv_heads, dim, vdim, splits):
    rng = np.random.default_rng(dim + splits)
    lens, bs = [1, 31, 33, 64, 130, 400], 32
    p = Pages(rng, lens, kv_heads, dim, vdim, bs, dtype)
    ctx = [1, 31, 2, 64, 129, 400, 333, 65, 0]                 # the last row is padding
    row_seq = [0, 1, 2, 3, 4, 5, 5, 4, 0]
    q = rounded(rng.standard_normal((len(ctx), heads, dim)), dtype)
    for r, (c, s) in enumerate(zip(ctx, row_seq)):
        # the last visible key stands out for head 0, the first invisible one would for the last head
        if c:
            q[r, 0] = 3 * p.k[s][c - 1, 0]
        if c < lens[s]:
            q[r, -1] = 3 * p.k[s][c, -1]
    q = rounded(q, dtype)
    scale, sink = 0.4 * dim ** -0.5, rng.standard_normal(heads) * 3
    gate = rounded(rng.standard_normal((len(ctx), heads + 3)), dtype)
    out = torch.full((len(ctx), heads * vdim + 4), 9.0, dtype=dtype, device=gpu)
    ho.grouped_attention(p.queries(q, dtype), dev(p.cache, dtype), dev(p.tables, torch.int32), dev(ctx, torch.int32), scale, vdim, out,
                         dev(sink), dev(gate, dtype), row_seq=dev(row_seq, torch.int32), splits=splits)
    want = np.zeros((len(ctx), heads, vdim))
    for r, (c, s) in enumerate(zip(ctx, row_seq)):
        if c:
            want[r] = one_query(q[r], p.k[s][:c], p.v[s][:c], scale, sink) * sigmoid(gate[r, :heads])[:, None]
    close(out[:, :heads * vdim], want.reshape(len(ctx), -1), tol(dtype, 3e-6, 1.5e-2))
    assert (out[:, heads * vdim:] == 9.0).all()
    # without sink and gate
    ho.grouped_attention(p.queries(q, dtype), dev(p.cache, dtype), dev(p.tables, torch.int32), dev(ctx, torch.int32), scale, vdim, out,
                         row_seq=dev(row_seq, torch.int32), splits=splits)
    plain = np.stack([one_query(q[r], p.k[s][:c], p.v[s][:c], scale, np.full(heads, -np.inf)) if c else np.zeros((heads, vdim))
                      for r, (c, s) in enumerate(zip(ctx, row_seq))])
    close(out[:, :heads * vdim], plain.reshape(len(ctx), -1), tol(dtype, 3e-6, 1.5e-2))


@BOTH
@pytest.mark.parametrize("sink", [-80.0, -3.0, 0.0, 4.0, 60.0, 300.0])
def test_a_sink_takes_its_share(gpu, dtype, sink):
    """Equal scores: with n keys every weight is e^s / (n e^s + e^sink), whatever splits the keys are cut into."""
    heads, dim, n, bs, score = 3, 32, 70, 32, 2.0
    p = Pages(np.random.default_rng(1), [n], 1, dim, dim, bs, dtype)
    p.cache[..., p.vp:] = np.where(np.isnan(p.cache[..., p.vp:]), np.nan, 1.0)
    p.cache[..., :p.vp] = np.where(np.isnan(p.cache[..., :p.vp]), np.nan, 1.0)
    q = np.full((1, heads, dim), score / dim)
    sinks = np.array([sink, -np.inf, sink])
    for splits in (1, 2):
        out = torch.empty((1, heads * dim), dtype=dtype, device=gpu)
        ho.grouped_attention(p.queries(q, dtype), dev(p.cache, dtype), dev(p.tables, torch.int32), dev([n], torch.int32), 1.0, dim, out,
                             dev(sinks), splits=splits)
        want = n * np.exp(score) / (n * np.exp(score) + np.exp(sinks))
        got = host(out).reshape(heads, dim)
        assert np.allclose(got, want[:, None], rtol=tol(dtype, 2e-6 + 1e-7 * abs(sink), 8e-3), atol=1e-30)


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(6, 2, 24, 16), (4, 1, 64, 64), (4, 4, 128, 128), (8, 2, 128, 64), (3, 1, 200, 96)])
def test_grouped_prefill(gpu, heads, kv_heads, dim, vdim):
    """Portions behind a cached prefix; keys at the edges of what a query sees stand out."""
    rng, bf = np.random.default_rng(dim), torch.bfloat16
    lens, new, bs = [130, 300, 64, 513], [130, 77, 64, 200], 64
    p = Pages(rng, lens, kv_heads, dim, vdim, bs, bf)
    assert ho.grouped_prefill_supported(dim, vdim)
    seqs = [2, 0, 3]
    cu_q, cu_k = np.cumsum([0] + [new[s] for s in seqs]), np.cumsum([0] + [lens[s] for s in seqs])
    q = [rounded(rng.standard_normal((new[s], heads, dim)), bf) for s in seqs]
    for x, s in zip(q, seqs):
        for i in range(0, len(x), 3):
            see = lens[s] - new[s] + i
            x[i, 0] = 2 * p.k[s][see, 0]                      # itself
            if see + 1 < lens[s]:
                x[i, -1] = 2 * p.k[s][see + 1, -1]            # the next token, invisible
            if i % 2:
                x[i, heads // 2] = 2 * p.k[s][0, heads // 2 // (heads // kv_heads)]
    q = [rounded(x, bf) for x in q]
    total_q = int(cu_q[-1])
    proj = torch.zeros((total_q, -(-(heads * dim + heads) // 8) * 8), dtype=bf, device=gpu)
    gate = rounded(rng.standard_normal((total_q, heads)), bf)
    proj[:, :heads * dim] = dev(np.concatenate(q).reshape(total_q, -1), bf)
    proj[:, heads * dim:heads * dim + heads] = dev(gate, bf)
    scale, sink = 0.5 * dim ** -0.5, rng.standard_normal(heads) * 3
    rows = ho.grouped_gather(dev(p.cache, bf), dev(p.tables, torch.int32), dev(seqs, torch.int32), dev(cu_k, torch.int32), int(cu_k[-1]), max(lens))
    out = torch.empty((total_q, heads * vdim), dtype=bf, device=gpu)
    want = np.zeros((total_q, heads, vdim))
    for i, s in enumerate(seqs):
        close(rows[cu_k[i]:cu_k[i + 1], :, p.vp:p.vp + dim], p.k[s], 0)
        close(rows[cu_k[i]:cu_k[i + 1], :, :vdim], p.v[s], 0)
    for use_sink in (True, False):
        ho.grouped_prefill(proj, rows[:, :, p.vp:], rows[:, :, :p.vp], dev(sink) if use_sink else None,
                           proj[:, heads * dim:heads * dim + heads], out, dev(cu_q, torch.int32), dev(cu_k, torch.int32),
                           max(new[s] for s in seqs), heads, dim, vdim, scale)
        for i, s in enumerate(seqs):
            for j in range(new[s]):
                see = lens[s] - new[s] + j + 1
                r = cu_q[i] + j
                want[r] = one_query(q[i][j], p.k[s][:see], p.v[s][:see], scale, sink if use_sink else np.full(heads, -np.inf))
        close(out, (want * sigmoid(gate)[..., None]).reshape(total_q, -1), 1.5e-2)


# ------------------------------------------------------------------ linear attention
class Decay:
    """One layer's inputs and what comes out, for several sequences."""
    KINDS = {"lightning": dict(silu=True, per_head=False, weight=True, gate_silu=False),
             "retention": dict(silu=False, per_head=True, weight=False, gate_silu=True),
             "plain": dict(silu=False, per_head=True, weight=True, gate_silu=False)}

    def __init__(self, kind, decay, dim, vdim, rot, dtype, seed=0, eps=1e-3):
        self.kind, self.decay, self.dim, self.vdim, self.dtype, self.eps = self.KINDS[kind], decay, dim, vdim, dtype, eps
        self.rng = np.random.default_rng(seed)
        self.heads, self.rot = len(decay), rot if kind == "retention" else 0
        k = self.kind
        self.scale = 1.0 if k["silu"] else 0.37
        self.shape = ho.DecayShape(self.heads, dim, vdim, eps, k["silu"], self.rot, self.scale, k["per_head"], k["gate_silu"])
        a, b = self.heads * dim, self.heads * vdim
        self.off = [0, a, 2 * a, 2 * a + b]
        self.off = [-(-o // 8) * 8 + 8 * i for i, o in enumerate(self.off)]
        self.cols = -(-(self.off[3] + b) // 8) * 8
        self.norm = 1 + .3 * self.rng.standard_normal(b) if k["weight"] else None
        self.table = yarn_rotary_table(self.rot, 8192, 300.0, None, "cuda") if self.rot else None

    def run(self, x, state, slots, positions, decode_rows, spans):
        out = torch.full((len(x), self.heads * self.vdim), float("nan"), dtype=self.dtype, device="cuda")
        ho.decay_attention(self.shape, dev(x, self.dtype), self.off, ho.decay_constants(self.decay, "cuda"), self.table,
                           dev(self.norm) if self.norm is not None else None, state, slots, positions, decode_rows,
                           dev(np.array(spans).reshape(-1, 4), torch.int32), max((s[1] for s in spans), default=0), out)
        return out

    def inputs(self, n):
        return rounded(self.rng.standard_normal((n, self.cols)), self.dtype)

    def want(self, x, pos0, state, round_silu=False):
        """Outputs and final states of one sequence's rows ``x`` from ``state`` [heads, dim, vdim]."""
        n, h = len(x), self.heads
        q, k = (x[:, o:o + h * self.dim].reshape(n, h, self.dim) for o in self.off[:2])
        v, g = (x[:, o:o + h * self.vdim].reshape(n, h, self.vdim) for o in self.off[2:])
        if self.kind["silu"]:
            q, k, v = silu(q), silu(k), silu(v)
            if round_silu:
                q, k, v = (rounded(a, torch.bfloat16) for a in (q, k, v))
        if self.rot:
            freq, _ = ref.yarn_frequencies(self.rot, 300.0)
            pos = pos0 + np.arange(n)
            q, k = ref.rotate_halves(q, pos, freq), ref.rotate_halves(k, pos, freq)
        o, end = np.zeros((n, h, self.vdim)), np.zeros((h, self.dim, self.vdim))
        for i in range(h):
            o[:, i], end[i] = ref.decay_scan(q[:, i], k[:, i], v[:, i], self.decay[i], state[i])
        o = o * self.scale
        w = 1.0 if self.norm is None else self.norm.reshape(h, self.vdim)
        if self.kind["per_head"]:
            o = rms_norm(o, w, self.eps)
        else:
            o = rms_norm(o.reshape(n, -1), 1.0, self.eps).reshape(o.shape) * w
        return (o * (silu(g) if self.kind["gate_silu"] else sigmoid(g))).reshape(n, -1), end

    def state(self, slots):
        s = self.shape
        return torch.full((slots, self.heads, s.state_rows, s.state_cols), float("nan"), device="cuda")

    def fill(self, state, slot, values):
        state[slot] = 0
        state[slot, :, :self.dim, :self.vdim] = dev(values)

    def check_state(self, state, slot, want, atol):
        got = state[slot]
        for i in range(self.heads):
            close(got[i, :self.dim, :self.vdim], want[i], atol)
        got = got.clone()
        got[:, :self.dim, :self.vdim] = 0
        assert not got.any()                                   # what pads the sizes stays zero


# name: decay, dim, vdim, rot
DECAYS = {
    "small": ((0.6, 0.97, 0.9995), 32, 32, 32), "uneven": ((0.9, 0.1), 48, 40, 32), "odd": ((0.95,), 10, 7, 6),
    "wide": ((0.97, 1.0 - 2.0 ** -12), 128, 128, 128), "narrow": ((0.99, 1e-30, 1.0), 16, 64, 16), "large": ((0.985,), 256, 256, 128),
    "long-v": ((0.7, 0.999), 64, 192, 64), "long-k": ((0.9,), 192, 16, 96), "odd-large": ((0.9,), 300, 100, 100),
}
BYKIND = pytest.mark.parametrize("kind", list(Decay.KINDS))
BYSIZE = pytest.mark.parametrize("size", list(DECAYS))


def state_tol(d, dtype):
    """float32 everywhere; silu is rounded to bf16 on the way in where the matrix pipe takes it."""
    return 6e-3 if d.kind["silu"] and dtype == torch.bfloat16 else 2e-6


@BOTH
@BYKIND
@BYSIZE
def test_decay_steps(gpu, dtype, kind, size):
    d = Decay(kind, *DECAYS[size], dtype)
    state = d.state(5)
    start = d.rng.standard_normal((d.heads, d.dim, d.vdim))
    d.fill(state, 3, start)                                    # sequence 0: under way in slot 3; sequence 1: new, slot 1 is NaN
    s0, s1 = start, np.zeros_like(start)
    for t in range(3):
        x = d.inputs(3)
        out = d.run(x, state, dev([3, -1, 1], torch.int32), dev([100 + t, 0, t], torch.int64), 3, [])
        w0, s0 = d.want(x[:1], 100 + t, s0)
        w1, s1 = d.want(x[2:], t, s1)
        close(out[:1], w0, tol(dtype, 5e-6))
        close(out[2:], w1, tol(dtype, 5e-6))
        assert not out[1].any()
    d.check_state(state, 3, s0, 2e-6)
    d.check_state(state, 1, s1, 2e-6)
    assert state[0].isnan().all() and state[2].isnan().all() and state[4].isnan().all()


@BOTH
@BYKIND
@BYSIZE
def test_decay_spans(gpu, dtype, kind, size):
    """Portions of several lengths, new and under way, with decoded tokens in front."""
    d = Decay(kind, *DECAYS[size], dtype, seed=5)
    counts = [2, 3, 31, 32, 33, 64, 100, 257]
    state = d.state(len(counts) + 2)
    decode = 2
    x = d.inputs(decode + sum(counts))
    spans, starts, at = [], [], decode
    for i, n in enumerate(counts):
        new = i % 2 == 0
        pos0 = 0 if new else 37 + i
        start = np.zeros((d.heads, d.dim, d.vdim)) if new else d.rng.standard_normal((d.heads, d.dim, d.vdim))
        if not new:
            d.fill(state, i + 2, start)
        spans.append((at, n, i + 2, pos0))
        starts.append(start)
        at += n
    out = d.run(x, state, dev([0, -1], torch.int32), dev([0, 0], torch.int64), decode, spans)
    close(out[:1], d.want(x[:1], 0, np.zeros_like(starts[0]))[0], tol(dtype, 2e-5))
    for (r, n, slot, pos0), start in zip(spans, starts):
        chunked = dtype == torch.bfloat16
        want, end = d.want(x[r:r + n], pos0, start, round_silu=chunked)
        close(out[r:r + n], want, tol(dtype, 1e-5))
        d.check_state(state, slot, end, state_tol(d, dtype))


@BYKIND
@pytest.mark.parametrize("n", [128, 1000, 3001])
def test_decay_segments(gpu, kind, n):
    """A long portion of few heads is cut into segments: a mark left by the first token is still there at the end."""
    bf = torch.bfloat16
    d = Decay(kind, (0.99951171875, 0.9, 1.0), 64, 64, 64, bf, seed=n)
    x = d.inputs(n) * 0.05
    x[0] *= 200.0
    x = rounded(x, bf)
    for pos0 in (0, 11):
        state = d.state(2)
        start = np.zeros((3, 64, 64)) if pos0 == 0 else d.rng.standard_normal((3, 64, 64))
        if pos0:
            d.fill(state, 1, start)
        out = d.run(x, state, None, None, 0, [(0, n, 1, pos0)])
        want, end = d.want(x, pos0, start, round_silu=True)
        close(out, want, 2e-2)
        d.check_state(state, 1, end, 6e-3 if kind == "lightning" else 3e-6)
        assert state[0].isnan().all()


@BYKIND
def test_decay_state_does_not_drift_over_many_steps(gpu, kind):
    """4000 decoded tokens of zeros: what is left of the state is decay^4000 of it to float precision."""
    d = Decay(kind, (1.0 - 1.1e-4, 0.9998), 32, 32, 32, torch.float32)
    state, start = d.state(1), d.rng.standard_normal((2, 32, 32))
    d.fill(state, 0, start)
    x = np.zeros((1, d.cols))
    args = [dev(x), d.off, ho.decay_constants(d.decay, "cuda"), d.table, dev(d.norm) if d.norm is not None else None, state,
            dev([0], torch.int32), dev([5], torch.int64), 1, None, 0, torch.empty((1, 64), device="cuda")]
    for _ in range(4000):
        ho.decay_attention(d.shape, *args)
    d.check_state(state, 0, start * (np.array(d.decay) ** 4000)[:, None, None], 2e-5)
