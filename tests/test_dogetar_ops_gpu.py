"""The kernels of masked attention, of the state space, of the mixture of experts and of the pre-norm residual stream, each alone,
against ``oracle/dogetar_ref.py`` (float64) on random inputs made so that a wrong key, token, state or expert shows."""
import numpy as np
import pytest
import torch

from infer_amd import hybrid_ops as ho, ops
from infer_amd.layers import banded_rotary_table
from oracle import dogetar_ref as ref
from oracle.merilorn_ref import rms_norm, sigmoid, silu
from tests.test_hybrid_ops_gpu import BOTH, close, dev, host, rounded, tol

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------ residual stream
@BOTH
@pytest.mark.parametrize("width", [8, 72, 129, 1000, 2563, 4096])
def test_pre_norm_forms(gpu, dtype, width):
    rng = np.random.default_rng(width)
    n, eps = 5, 1e-2
    x0, first = rng.standard_normal((2, n, width))
    y = rounded(rng.standard_normal((n, width)) * .3, dtype)
    w, scale, step = 1 + rng.standard_normal((3, width)) * .3
    t = tol(dtype, 2e-6, 8e-3)
    for kw, want in ((dict(), x0 + y), (dict(scale=scale), x0 + y * scale), (dict(scale=scale, step=step), x0 + y * scale + step),
                     (dict(scale=scale, step=step, first=first), x0 + y * scale + first + step)):
        x = dev(x0)
        h = ho.pre_norm(x, dev(w), eps, y=dev(y, dtype), dtype=dtype, **{k: dev(v) for k, v in kw.items()})
        close(x, want, 2e-6)
        close(h, rms_norm(want, w, eps), t)


@BOTH
@pytest.mark.parametrize("width", [16, 77])
def test_embedding_of_tokens_and_pairs(gpu, dtype, width):
    rng = np.random.default_rng(width)
    buckets, mul_prev, mul_cur, vocab = 13, 2 ** 20 + 7, 5, 11
    embed, bigram = rounded(rng.standard_normal((vocab, width)), dtype), rounded(rng.standard_normal((buckets + 1, width)), dtype)
    seqs = [[3, 0, 10, 10, 7], [4], [9, 1]]
    ids, prev = np.concatenate(seqs), np.concatenate([[-1] + s[:-1] for s in seqs])
    want = np.concatenate([embed[s] + bigram[ref.bigram_rows(s, buckets, mul_prev, mul_cur)] for s in seqs])
    w, step = 1 + rng.standard_normal((2, width)) * .2
    x, first = torch.full((8, width), float("nan"), device=gpu), torch.full((8, width), float("nan"), device=gpu)
    h = ho.pre_norm(x, dev(w), 1e-3, tokens=dev(ids, torch.int64), embed=dev(embed, dtype), prev=dev(prev, torch.int64),
                    bigram=dev(bigram, dtype), multipliers=(mul_prev, mul_cur), first=first, step=dev(step), dtype=dtype)
    close(first, want, 1e-6)
    close(x, want + step, 1e-6)
    close(h, rms_norm(want + step, w, 1e-3), tol(dtype, 2e-6, 8e-3))


@BOTH
@pytest.mark.parametrize("split_k", [False, True])
def test_pre_norm_sums_experts(gpu, dtype, split_k):
    rng = np.random.default_rng(3)
    n, width, top, places = 6, 512, 3, 11
    rows, h = rounded(rng.standard_normal((places, width)), dtype), rounded(rng.standard_normal((n, width)), dtype)
    at, wt = rng.integers(-1, places, (n, top)).astype(np.int32), rng.random((n, top))
    x0, scale, w = rng.standard_normal((n, width)), rng.standard_normal(width), 1 + .1 * rng.standard_normal(width)
    shared = dev(rng.standard_normal((n, width)), dtype)
    if split_k:
        if dtype == torch.float32:
            pytest.skip("split-K products are bfloat16")
        shared = ops.linear(dev(rng.standard_normal((n, 4096)), dtype), dev(rng.standard_normal((width, 4096)) * .02, dtype), defer=True)
        assert isinstance(shared, ops.SplitKSum)
    value = host(shared.partial).sum(0) if split_k else host(shared)
    for s, v in ((None, 0.0), (shared, value)):
        y = v + sum(wt[:, k, None] * np.where(at[:, k, None] < 0, h, rows[np.maximum(at[:, k], 0)]) for k in range(top))
        x = dev(x0)
        ho.pre_norm(x, dev(w), 1e-6, y=ho.ExpertSum(dev(rows, dtype), dev(at, torch.int32), dev(wt), dev(h, dtype), s), scale=dev(scale), dtype=dtype)
        close(x, x0 + y * scale, 2e-6)


@BOTH
@pytest.mark.parametrize("d", [8, 30, 352])
def test_clamped_gate(gpu, dtype, d):
    x = rounded(np.random.default_rng(d).standard_normal((6, 2 * d)) * 3, dtype)
    x[0, 0], x[1, 0], x[2, d], x[3, d] = 60.0, -60.0, 40.0, -40.0
    g, u = np.minimum(x[:, :d], 1.5), np.clip(x[:, d:], -1.5, 1.5)
    close(ho.clamped_gate_and_mul(dev(x, dtype), 1.5), g * sigmoid(1.702 * g) * (u + 1.0), tol(dtype, 1e-6, 4e-3))


@BOTH
def test_softcap(gpu, dtype):
    x = rounded(np.random.default_rng(0).standard_normal((3, 1031)) * 40, dtype)
    got = ho.softcap(dev(x, dtype), 7.5)
    assert got.dtype == torch.float32
    close(got, 7.5 * np.tanh(x / 7.5), 1e-6)


# ------------------------------------------------------------------ masked attention
def offsets_of(s, gap=5):
    q = 8
    k = q + -(-s.heads * s.maps * s.dim // 8) * 8
    v = k + -(-s.kv_heads * s.maps * s.dim // 8) * 8
    cols = v + s.kv_heads * s.vdim + gap
    return [q, k, v], cols + -cols % 8


@BOTH
@pytest.mark.parametrize("heads,kv_heads,maps,dim,vdim,rot", [(6, 2, 1, 24, 16, 16), (4, 4, 2, 32, 64, 32), (3, 1, 1, 10, 7, 4), (5, 5, 2, 9, 8, 6),
                                                              (16, 2, 1, 128, 128, 64), (32, 8, 2, 64, 128, 64), (8, 1, 1, 64, 32, 0),
                                                              (2, 1, 1, 200, 40, 200), (40, 8, 1, 128, 128, 128), (6, 3, 2, 48, 96, 16)])
@pytest.mark.parametrize("extras", [True, False], ids=["bias-norm", "plain"])
def test_head_front(gpu, dtype, heads, kv_heads, maps, dim, vdim, rot, extras):
    rng = np.random.default_rng(heads * dim)
    n, bs, nblk, qx_rows = 7, 32, 3, 3
    s = ho.MaskedShape(heads, kv_heads, dim, vdim, 1.0, maps=maps, eps=1e-2, rot_dims=rot)
    off, cols = offsets_of(s)
    x = rounded(rng.standard_normal((n, cols)), dtype)
    bias, (qn, kn) = rng.standard_normal(cols), 1 + .3 * rng.standard_normal((2, dim))
    pos, slots = rng.integers(0, 200, n), np.array([5, 31, 32, -1, 64, 95, 200], np.int32)      # one padding row, one outside the pool
    r = {"base": 77.0, "dims": rot, "scaling": dict(factor=3.0, original=64, low=1.0, high=4.0)}
    table = banded_rotary_table(rot, 256, r["base"], r["scaling"], gpu) if rot else None
    cache = torch.full((nblk, kv_heads, bs, s.vdim_pad + s.key_pad), 7.0, dtype=dtype, device=gpu)
    qx = torch.full((qx_rows, heads * maps, s.key_pad), float("nan"), dtype=dtype, device=gpu)
    proj = dev(x, dtype)
    ho.head_front(s, proj, off, dev(bias) if extras else None, dev(qn) if extras else None, dev(kn) if extras else None, table,
                  dev(pos, torch.int64), dev(slots, torch.int32), cache, qx, qx_rows)
    y = x + bias if extras else x

    def turned(at, h, w):
        z = y[:, at:at + h * maps * dim].reshape(n, h, maps, dim)
        z = rms_norm(z, w, 1e-2) if extras else z
        return ref.rotate_halves(z, pos, ref.scaled_frequencies(r)) if rot else z

    q, k = turned(off[0], heads, qn), turned(off[1], kv_heads, kn)
    v = y[:, off[2]:off[2] + kv_heads * vdim].reshape(n, kv_heads, vdim)
    t = tol(dtype, 2e-6, 8e-3)
    padded = np.zeros((qx_rows, heads, maps, s.key_pad))
    for i in range(maps):
        padded[:, :, i, i * dim:(i + 1) * dim] = q[:qx_rows, :, i]
    close(qx, padded.reshape(qx.shape), t)
    width = heads * maps * dim
    close(proj[qx_rows:, off[0]:off[0] + width], q[qx_rows:].reshape(n - qx_rows, -1), t)
    left = np.r_[0:off[0], off[0] + width:cols]
    assert np.array_equal(host(proj[:qx_rows]), x[:qx_rows]) and np.array_equal(host(proj)[:, left], x[:, left])
    got = host(cache).transpose(0, 2, 1, 3).reshape(nblk * bs, kv_heads, -1)
    for i, slot in enumerate(slots):
        if 0 <= slot < nblk * bs:
            want = np.zeros(got[slot].shape)
            want[:, :vdim] = v[i]
            want[:, s.vdim_pad:s.vdim_pad + maps * dim] = k[i].reshape(kv_heads, -1)
            close(torch.tensor(got[slot]), want, t)
    assert (got[[i for i in range(nblk * bs) if i not in slots]] == 7.0).all()


class Pages:
    """Random keys and values of several sequences in shuffled pages; every row that belongs to nobody is NaN."""

    def __init__(self, rng, lens, s, bs, dtype):
        self.s = s
        self.k = [rounded(rng.standard_normal((n, s.kv_heads, s.maps, s.dim)), dtype) for n in lens]
        self.v = [rounded(rng.standard_normal((n, s.kv_heads, s.vdim)), dtype) for n in lens]
        counts = [-(-n // bs) for n in lens]
        self.tables = np.full((len(lens), max(counts) + 1), -1, np.int32)
        ids = rng.permutation(sum(counts) + 2)
        cache = np.full((sum(counts) + 2, s.kv_heads, bs, s.vdim_pad + s.key_pad), np.nan)
        at = 0
        for i, n in enumerate(lens):
            for b in range(counts[i]):
                block = self.tables[i, b] = ids[at]
                at += 1
                m = min(bs, n - b * bs)
                rows = cache[block, :, :m]
                rows[:] = 0.0
                rows[..., :s.vdim] = self.v[i][b * bs:b * bs + m].transpose(1, 0, 2)
                rows[..., s.vdim_pad:s.vdim_pad + s.maps * s.dim] = self.k[i][b * bs:b * bs + m].reshape(m, s.kv_heads, -1).transpose(1, 0, 2)
        self.cache, self.tables = dev(cache, dtype), dev(self.tables, torch.int32)


def first_seen(s, pos):
    return 0 if s.mask is None else pos // s.mask_size * s.mask_size if s.mask == "chunk" else max(0, pos - s.mask_size + 1)


def one_query(s, q, k, v, pos, sink, gate):
    """``q`` [heads, maps, dim] at position ``pos`` over the keys 0 .. pos."""
    lo, group = first_seen(s, pos), s.heads // s.kv_heads
    out = np.zeros((s.maps, s.heads, s.vdim))
    for m in range(s.maps):
        for h in range(s.heads):
            z = k[lo:pos + 1, h // group, m] @ q[h, m] * s.scale
            if s.distance_bias:
                z = z - 2.0 ** (-8.0 * (h + 1) / s.heads) * (pos - np.arange(lo, pos + 1))
            top = max(z.max(), sink[h])
            p = np.exp(z - top)
            out[m, h] = p @ v[lo:pos + 1, h // group] / (p.sum() + np.exp(sink[h] - top))
    o = out[0] if s.maps == 1 else rms_norm(out[0] - s.lam * out[1], 1.0, s.eps)
    return o * s.out_scale * sigmoid(gate)[:, None]


MASKS = [(None, 1), ("chunk", 1), ("chunk", 33), ("chunk", 96), ("window", 1), ("window", 31), ("window", 64), ("window", 100), ("window", 5000)]
SHAPES = [(6, 2, 24, 16, 1), (1, 1, 10, 7, 1), (32, 4, 128, 128, 1), (40, 2, 96, 32, 1), (4, 2, 320, 300, 1), (6, 2, 24, 40, 2), (4, 4, 64, 128, 2),
          (5, 1, 9, 11, 2), (2, 1, 128, 200, 2)]


def standing_out(rng, s, p, i, pos, dtype, lens):
    """A query for whose heads the edge keys of what it sees stand out: the first seen, the last seen, and invisible neighbours."""
    q = rng.standard_normal((s.heads, s.maps, s.dim))
    lo, group = first_seen(s, pos), s.heads // s.kv_heads
    for h, at in zip(range(s.heads), (lo, pos, lo - 1, pos + 1)):
        if 0 <= at < lens[i]:
            q[h] = 3 * p.k[i][at, h // group] / (s.dim * s.scale / 4)
    return rounded(q, dtype)


@BOTH
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,maps", SHAPES)
@pytest.mark.parametrize("mask,size", MASKS)
def test_masked_attention_rows(gpu, dtype, heads, kv_heads, dim, vdim, maps, mask, size):
    rng = np.random.default_rng(dim + size)
    s = ho.MaskedShape(heads, kv_heads, dim, vdim, 0.4 * dim ** -0.5, maps=maps, mask=mask, mask_size=size, distance_bias=maps == 1,
                       out_scale=0.6, lam=0.7, eps=1e-3)
    lens, bs = [1, 31, 33, 64, 130, 330], 32
    p = Pages(rng, lens, s, bs, dtype)
    ctx = [1, 31, 2, 64, 129, 330, 32, 193, 65, 0]             # the last row is padding
    row_seq = [0, 1, 2, 3, 4, 5, 4, 5, 4, 0]
    q = np.stack([standing_out(rng, s, p, i, max(c - 1, 0), dtype, lens) for c, i in zip(ctx, row_seq)])
    sink, gate = rng.standard_normal(heads) * 3, rounded(rng.standard_normal((len(ctx), heads + 3)), dtype)
    none = np.full(heads, -np.inf)
    qx = np.zeros((len(ctx), heads, maps, s.key_pad))
    for m in range(maps):
        qx[:, :, m, m * dim:(m + 1) * dim] = q[:, :, m]
    args = (dev(qx.reshape(len(ctx), heads * maps, -1), dtype), p.cache, p.tables, dev(ctx, torch.int32))
    for splits in (0, 1, 3):
        for full in (True, False):
            out = torch.full((len(ctx), heads * vdim + 4), 9.0, dtype=dtype, device=gpu)
            ho.masked_attention(s, *args, out, dev(sink) if full and maps == 1 else None, dev(gate, dtype) if full else None,
                                row_seq=dev(row_seq, torch.int32), splits=splits)
            want = np.zeros((len(ctx), heads, vdim))
            for r, (c, i) in enumerate(zip(ctx, row_seq)):
                if c:
                    want[r] = one_query(s, q[r], p.k[i], p.v[i], c - 1, sink if full and maps == 1 else none,
                                        gate[r, :heads] if full else np.full(heads, np.inf))
            close(out[:, :heads * vdim], want.reshape(len(ctx), -1), tol(dtype, 1e-5, 2e-2))
            assert (out[:, heads * vdim:] == 9.0).all()


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,maps", [(6, 2, 24, 16, 1), (4, 4, 128, 128, 1), (3, 1, 200, 96, 1), (6, 2, 24, 40, 2), (4, 2, 64, 128, 2),
                                                          (2, 1, 72, 64, 2)])
@pytest.mark.parametrize("mask,size", MASKS)
def test_masked_prefill(gpu, heads, kv_heads, dim, vdim, maps, mask, size):
    """Portions behind a cached prefix; keys at the edges of what a query sees stand out, rows nobody sees are NaN."""
    rng, bf = np.random.default_rng(dim + size), torch.bfloat16
    s = ho.MaskedShape(heads, kv_heads, dim, vdim, 0.5 * dim ** -0.5, maps=maps, mask=mask, mask_size=size, distance_bias=maps == 1,
                       out_scale=0.6, lam=0.7, eps=1e-3)
    assert ho.masked_prefill_supported(s)
    lens, new = [130, 300, 64, 413], [130, 77, 64, 200]
    p = Pages(rng, lens, s, 64, bf)
    seqs = [2, 0, 3]
    cu_q, cu_k = np.cumsum([0] + [new[i] for i in seqs]), np.cumsum([0] + [lens[i] for i in seqs])
    q = np.concatenate([np.stack([standing_out(rng, s, p, i, lens[i] - new[i] + t, bf, lens) if t % 3 else rounded(
        rng.standard_normal((heads, maps, dim)), bf) for t in range(new[i])]) for i in seqs])
    total = int(cu_q[-1])
    proj = torch.zeros((total, 8 + -(-(heads * maps * dim + heads) // 8) * 8), dtype=bf, device=gpu)
    gate, sink = rounded(rng.standard_normal((total, heads)), bf), rng.standard_normal(heads) * 3
    proj[:, 8:8 + heads * maps * dim] = dev(q.reshape(total, -1), bf)
    cu = dev(cu_q, torch.int32), dev(cu_k, torch.int32)
    rows = torch.full((int(cu_k[-1]), kv_heads, s.vdim_pad + s.key_pad), float("nan"), dtype=bf, device=gpu)
    del rows                                                     # the gather's own buffer likely reuses it
    rows = ho.masked_gather(s, p.cache, p.tables, dev(seqs, torch.int32), *cu, int(cu_k[-1]), max(lens[i] for i in seqs))
    for full in (True, False):
        out = torch.empty((total, heads * vdim), dtype=bf, device=gpu)
        ho.masked_prefill(s, proj[:, 8:], rows, out, *cu, max(new[i] for i in seqs), dev(sink) if full and maps == 1 else None,
                          dev(gate, bf) if full else None)
        want = np.zeros((total, heads, vdim))
        for j, i in enumerate(seqs):
            for t in range(new[i]):
                r = int(cu_q[j]) + t
                want[r] = one_query(s, q[r], p.k[i], p.v[i], lens[i] - new[i] + t, sink if full and maps == 1 else np.full(heads, -np.inf),
                                    gate[r] if full else np.full(heads, np.inf))
        close(out, want.reshape(total, -1), 2e-2)


# ------------------------------------------------------------------ state space
class Ssm:
    """Random weights of a layer, and sequences that are fed to it in portions."""

    def __init__(self, rng, shape, dtype, slots=5, a_log=(-5.0, 1.5), dt=1.0):
        self.s = s = ho.StateSpaceShape(*shape, eps=1e-3)
        self.dtype, self.rng = dtype, rng
        self.conv, self.conv_b = rng.standard_normal((s.channels, s.taps)) * s.taps ** -0.5, rng.standard_normal(s.channels) * .3
        self.dt_bias, self.d = rng.standard_normal(s.heads) * dt, rng.standard_normal(s.heads)
        self.a_log, self.norm = rng.uniform(*a_log, s.heads), 1 + .2 * rng.standard_normal(s.inner)
        self.ring = torch.full((slots, s.taps, s.channels), float("nan"), dtype=dtype, device="cuda")
        self.state = torch.full((slots, s.heads, s.state, s.vdim), float("nan"), device="cuda")
        self.off = (8, 8 + s.inner, 8 + s.inner + s.channels)
        self.cols = -(-(self.off[2] + s.heads) // 8) * 8

    def inputs(self, n):
        return rounded(self.rng.standard_normal((n, self.cols)), self.dtype)

    def want(self, x, cast=lambda a: a):
        """Outputs and final states of one whole sequence; ``cast`` is applied behind the convolution and to what the norm gets."""
        s = self.s
        z, xbc, dt = (x[:, a:b] for a, b in ((self.off[0], self.off[1]), (self.off[1], self.off[2]), (self.off[2], self.off[2] + s.heads)))
        xbc = cast(silu(ref.causal_conv(xbc, self.conv, self.conv_b)))
        dt = ref.softplus(dt + self.dt_bias)
        n, y, states = len(x), np.zeros((len(x), s.heads, s.vdim)), []
        b = xbc[:, s.inner:s.inner + s.groups * s.state].reshape(n, s.groups, s.state)
        c = xbc[:, s.inner + s.groups * s.state:].reshape(n, s.groups, s.state)
        for h in range(s.heads):
            g = h // (s.heads // s.groups)
            y[:, h], st = ref.state_space_scan(xbc[:, h * s.vdim:(h + 1) * s.vdim], b[:, g], c[:, g], dt[:, h], -np.exp(self.a_log[h]), self.d[h])
            states.append(st)
        return ref.gated_part_norm(cast(y.reshape(n, -1)), z, s.norm_parts, self.norm, s.eps), np.stack(states)

    def run(self, portions):
        """``portions``: (slot, first position, rows), decoded tokens first.  One step; the outputs in that order."""
        x = np.concatenate([rows for _, _, rows in portions])
        n, decode = len(x), sum(len(rows) == 1 for _, _, rows in portions)
        pos = np.concatenate([lo + np.arange(len(rows)) for _, lo, rows in portions])
        starts = np.cumsum([0] + [len(rows) for _, _, rows in portions])
        spans = [(starts[i], len(rows), slot, lo) for i, (slot, lo, rows) in enumerate(portions) if len(rows) > 1]
        ring_slot = np.concatenate([[(slot, len(rows) - 1 - j) for j in range(len(rows))] for slot, _, rows in portions])
        out = torch.full((n, self.s.inner + 8), 9.0, dtype=self.dtype, device="cuda")
        ho.state_space(self.s, dev(x, self.dtype), self.off, dev(self.conv), dev(self.conv_b), dev(self.dt_bias), dev(self.a_log), dev(self.d),
                       dev(self.norm), self.ring, self.state, dev([slot for slot, _, rows in portions if len(rows) == 1], torch.int32),
                       dev(pos, torch.int64), decode, dev(np.reshape(spans, (-1, 4)), torch.int32), max([c for _, c, _, _ in spans], default=0),
                       dev(ring_slot, torch.int32), out[:, :self.s.inner])
        assert (out[:, self.s.inner:] == 9.0).all()
        return np.split(host(out[:, :self.s.inner]), starts[1:-1])


# heads, vdim, state, groups, taps, parts
SSM = [(4, 16, 24, 2, 4, 2), (1, 6, 5, 1, 3, 2), (4, 64, 128, 2, 4, 2), (3, 72, 64, 1, 4, 1), (2, 136, 256, 2, 2, 4), (6, 8, 16, 3, 1, 3), (2, 12, 300, 1, 5, 1)]
CUTS = [[97], [1] * 97, [2] * 10 + [33, 3, 1, 1, 40], [64, 33], [5, 1, 91], [31, 66]]


@BOTH
@pytest.mark.parametrize("shape", SSM)
def test_state_space_however_it_is_cut(gpu, dtype, shape):
    m = Ssm(np.random.default_rng(sum(shape)), shape, dtype)
    x = m.inputs(97)
    want, states = m.want(x)
    for i, cuts in enumerate(CUTS):
        lo, got, slot = 0, [], i % 5
        for c in cuts:
            got += m.run([(slot, lo, x[lo:lo + c])])
            lo += c
        close(torch.tensor(np.concatenate(got)), want, tol(dtype, 1e-5, 2e-2))
        close(m.state[slot], states, tol(dtype, 1e-5, 1e-2))


@BOTH
def test_state_space_of_unequal_sequences_in_one_step(gpu, dtype):
    m = Ssm(np.random.default_rng(1), SSM[0], dtype)
    x = [m.inputs(n) for n in (70, 45, 33, 100)]
    want = [m.want(a)[0] for a in x]
    steps = [[(0, 0, 20), (1, 0, 2), (2, 0, 33)], [(0, 20, 1), (3, 0, 40), (1, 2, 43)], [(0, 21, 1), (3, 40, 60)], [(0, 22, 48)]]
    for step in steps:
        step = sorted(step, key=lambda p: p[2] > 1)
        got = m.run([(4 - i, lo, x[i][lo:lo + c]) for i, lo, c in step])
        for (i, lo, c), y in zip(step, got):
            close(torch.tensor(y), want[i][lo:lo + c], tol(dtype, 1e-5, 2e-2))


@pytest.mark.parametrize("shape", [SSM[2], SSM[3]])
def test_state_space_segments_of_a_long_portion(gpu, shape):
    """Few heads and one sequence: the portion is cut into segments whose states are joined."""
    m = Ssm(np.random.default_rng(5), shape, torch.bfloat16, a_log=(-9.0, -5.0))           # a memory of thousands of tokens
    x = m.inputs(1333)
    want, states = m.want(x)
    got = m.run([(2, 0, x[:1000])]) + m.run([(2, 1000, x[1000:])])
    close(torch.tensor(np.concatenate(got)), want, 2e-2)
    close(m.state[2], states, 1e-2)


@BOTH
@pytest.mark.parametrize("a_log,dt", [((4.0, 9.0), 3.0), ((-20.0, -12.0), 1.0), ((-1.0, 0.0), 12.0)])
def test_state_space_extreme_decays(gpu, dtype, a_log, dt):
    """Total loss from token to token, none at all, and step sizes from 0 to 20 side by side.  Large steps enlarge what
    rounding does to small products of B and C, so the limit is a multiple of that."""
    m = Ssm(np.random.default_rng(7), SSM[0], dtype, a_log=a_log, dt=dt)
    x = m.inputs(97)
    want, states = m.want(x)
    alone = np.abs(m.want(x, lambda a: rounded(a, torch.bfloat16))[0] - want).max() / np.abs(want).max()
    for slot, cuts in enumerate(([97], [1] * 97, [40, 57])):
        lo, got = 0, []
        for c in cuts:
            got += m.run([(slot, lo, x[lo:lo + c])])
            lo += c
        close(torch.tensor(np.concatenate(got)), want, tol(dtype, 2e-5, max(2e-2, 2 * alone)))
        close(m.state[slot], states, tol(dtype, 2e-5, 1e-2))


def test_state_keeps_float_precision_in_bfloat16(gpu):
    """Inputs that are powers of two and taps that hand them on: what enters the state has no bf16 rounding in it."""
    m = Ssm(np.random.default_rng(2), (2, 16, 32, 1, 1, 1), torch.bfloat16, a_log=(-8.0, -6.0))
    m.conv[:], m.conv_b[:] = 0.0, 3.0                         # x, B and C are silu(3), rounded once
    x = m.inputs(200)
    m.run([(0, 0, x)])
    dt = ref.softplus(x[:, m.off[2]:m.off[2] + 2] + m.dt_bias)
    unit = float(rounded(silu(np.array(3.0)), torch.bfloat16)) ** 2
    want = np.zeros(2)
    for t in range(200):
        want = np.exp(-np.exp(m.a_log) * dt[t]) * want + dt[t] * unit
    got = host(m.state[0])
    assert np.allclose(got, want[:, None, None], rtol=2e-6)


# ------------------------------------------------------------------ mixture of experts
# width, ff, experts, top, identity, groups, keep
MOE = [(64, 24, 5, 2, 1, 3, 2), (50, 9, 3, 1, 0, 1, 1), (128, 64, 8, 2, 0, 4, 2), (320, 136, 40, 6, 8, 8, 3), (256, 96, 60, 8, 4, 1, 1), (36, 20, 2, 4, 2, 1, 1),
       (96, 40, 200, 3, 56, 16, 4)]


@BOTH
@pytest.mark.parametrize("width,ff,experts,top,identity,groups,keep", MOE)
@pytest.mark.parametrize("n", [1, 17, 300])
def test_moe(gpu, dtype, width, ff, experts, top, identity, groups, keep, n):
    rng = np.random.default_rng(width + n)
    s = ho.MoeShape(width, ff, experts, top, identity, groups, keep, 1.7)
    every = experts + identity
    router = rounded(rng.standard_normal((every, width)) * 2 * width ** -0.5, dtype)
    correction = rng.standard_normal(every) * .1 - .2          # choice scores on both sides of zero
    gate, up = rounded(rng.standard_normal((2, experts, ff, width)) * width ** -0.5, dtype)
    down = rounded(rng.standard_normal((experts, width, ff)) * ff ** -0.5, dtype)
    # tokens whose choice is no close call
    pool = rounded(rng.standard_normal((40 * n, width)), dtype)
    z = pool @ router.T
    calls = [ref.route(z + e * rng.standard_normal(z.shape), correction, top, {"count": groups, "keep": keep}, 1.7)[0] for e in (0, 3e-4, 3e-4, 3e-4)]
    h = pool[[i for i in range(len(pool)) if all(np.array_equal(calls[0][i], c[i]) for c in calls[1:])][:n]]
    assert len(h) == n
    w = {"router": router, "correction": correction}
    for e in range(experts):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = gate[e], up[e], down[e]
    want = ref.mixture(h, {"router": {"experts": experts, "identity": identity, "top": top, "scale": 1.7, "groups": {"count": groups, "keep": keep}}}, w.get)
    padded = np.zeros((experts, width, s.ff_pad))
    padded[..., :ff] = down
    counts = torch.zeros(experts, dtype=torch.int32, device=gpu)
    lead = dev(np.concatenate([h, np.zeros((n, 8))], 1), dtype)[:, :width]
    for _ in range(2):                                         # the counters are clean again behind a step
        r = ho.moe(s, lead, dev(router, dtype), dev(correction), dev(np.concatenate([gate, up], 1), dtype), dev(padded, dtype), counts)
        x = torch.zeros((n, width), device=gpu)
        ho.pre_norm(x, torch.ones(width, device=gpu), 1e-6, y=r, dtype=dtype)
        close(x, want, tol(dtype, 1e-5, 2e-2))
        assert not counts.any()
    places = host(r.places)
    assert sorted(places[places >= 0]) == list(range((places >= 0).sum()))
    chosen, weight = ref.route(h @ router.T, correction, top, {"count": groups, "keep": keep}, 1.7)
    close(r.weights, weight, 1e-5)
    assert np.array_equal(places < 0, chosen >= experts)


@pytest.mark.parametrize("width,ff,experts,top", [(128, 64, 2, 1), (192, 320, 3, 2), (64, 100, 4, 1)])
def test_moe_of_many_rows_per_expert(gpu, width, ff, experts, top):
    """Rows enough for the largest blocks, unequal numbers of them, blocks that are nearly empty; both products and every row's place.
    The last case pads the inner width to no multiple of the large blocks' step."""
    rng, n, bf = np.random.default_rng(ff), 2500, torch.bfloat16
    s = ho.MoeShape(width, ff, experts, top, 0, 1, 1, 1.5)
    router, correction = rounded(rng.standard_normal((experts, width)) * 2 * width ** -0.5, bf), np.linspace(-0.15, 0.2, experts)
    gate, up = rounded(rng.standard_normal((2, experts, ff, width)) * width ** -0.5, bf)
    down = rounded(rng.standard_normal((experts, width, ff)) * ff ** -0.5, bf)
    pool = rounded(rng.standard_normal((4 * n, width)), bf)
    p = np.exp(pool @ router.T)
    choice = np.sort(p / p.sum(-1, keepdims=True) + correction, -1)
    h = pool[choice[:, -top] - choice[:, -top - 1] > 2e-3][:n]
    assert len(h) == n
    w = {"router": router, "correction": correction}
    for e in range(experts):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = gate[e], up[e], down[e]
    want = ref.mixture(h, {"router": {"experts": experts, "top": top, "scale": 1.5}}, w.get)
    padded = np.zeros((experts, width, s.ff_pad))
    padded[..., :ff] = down
    counts = torch.zeros(experts, dtype=torch.int32, device=gpu)
    weights = dev(router, bf), dev(correction), dev(np.concatenate([gate, up], 1), bf), dev(padded, bf), counts
    r = ho.moe(s, dev(h, bf), *weights)
    x = torch.zeros((n, width), device=gpu)
    ho.pre_norm(x, torch.ones(width, device=gpu), 1e-6, y=r)
    close(x, want, 2e-2)
    assert not counts.any()
    few = ho.moe(s, dev(h[:70], bf), *weights)                 # other kernels: a token's result does not depend on the batch
    y = torch.zeros((70, width), device=gpu)
    ho.pre_norm(y, torch.ones(width, device=gpu), 1e-6, y=few)
    close(y, host(x[:70]), 1e-2)


def test_moe_when_all_tokens_want_the_same_expert(gpu):
    rng, n, width, experts = np.random.default_rng(0), 700, 64, 6
    s = ho.MoeShape(width, 32, experts, 1, 0, 1, 1, 1.0)
    w = [rounded(rng.standard_normal(shape) * .1, torch.bfloat16) for shape in ((experts, width), (experts, 64, width), (experts, width, 32))]
    h = rounded(rng.standard_normal((n, width)), torch.bfloat16)
    correction = np.where(np.arange(experts) == 4, 2.0, 0.0)
    r = ho.moe(s, dev(h, torch.bfloat16), dev(w[0], torch.bfloat16), dev(correction), dev(w[1], torch.bfloat16), dev(w[2], torch.bfloat16),
               torch.zeros(experts, dtype=torch.int32, device=gpu))
    p = np.exp(h @ w[0].T)
    y = (silu(h @ w[1][4][:32].T) * (h @ w[1][4][32:].T)) @ w[2][4].T
    x = torch.zeros((n, width), device=gpu)
    ho.pre_norm(x, torch.ones(width, device=gpu), 1e-6, y=r, dtype=torch.bfloat16)
    close(x, y * (p[:, 4] / p.sum(-1))[:, None], 2e-2)


def test_bad_arguments_are_refused(gpu):
    z = torch.zeros(8, 64, device=gpu)
    counts = torch.zeros(4, dtype=torch.int32, device=gpu)
    with pytest.raises(RuntimeError):                          # five of four experts
        ho.moe(ho.MoeShape(64, 8, 4, 5), z, torch.zeros(4, 64, device=gpu), None, torch.zeros(4, 16, 64, device=gpu), torch.zeros(4, 64, 8, device=gpu), counts)
    s = ho.MaskedShape(2, 1, 16, 16, 1.0, maps=2, distance_bias=True)
    with pytest.raises(RuntimeError):                          # two maps have no bias
        ho.masked_attention(s, torch.zeros(1, 4, 32, device=gpu), torch.zeros(1, 1, 32, 64, device=gpu), torch.zeros(1, 1, dtype=torch.int32, device=gpu),
                            torch.ones(1, dtype=torch.int32, device=gpu), torch.zeros(1, 32, device=gpu))
    with pytest.raises(RuntimeError):                          # a mask that shows nothing
        ho.masked_attention(ho.MaskedShape(2, 1, 16, 16, 1.0, mask="window", mask_size=0), torch.zeros(1, 2, 32, device=gpu),
                            torch.zeros(1, 1, 32, 64, device=gpu), torch.zeros(1, 1, dtype=torch.int32, device=gpu),
                            torch.ones(1, dtype=torch.int32, device=gpu), torch.zeros(1, 32, device=gpu))
