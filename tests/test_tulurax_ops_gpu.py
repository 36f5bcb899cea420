"""The kernels of talking-heads attention, of the squashing norm and of the learned activation, each alone, against
``oracle/tulurax_ref.py`` (float64) on random inputs made so that a wrong key, head or token shows."""
import numpy as np
import pytest
import torch

from infer_amd import hybrid_ops as ho, ops
from oracle import tulurax_ref as ref
from oracle.merilorn_ref import rms_norm
from tests.test_hybrid_ops_gpu import BOTH, close, dev, host, rounded, tol

pytestmark = pytest.mark.gpu


# ------------------------------------------------------------------ residual stream, activation, logits
def tanh_parts(rng, width):
    alpha, w, b = float(rng.uniform(0.3, 1.2)), 1 + rng.standard_normal(width) * .3, rng.standard_normal(width) * .4
    return (alpha, w, b), ho.TanhNorm(alpha, dev(w), dev(b))


@BOTH
@pytest.mark.parametrize("rows,width", [(5, 8), (5, 72), (5, 129), (3, 1000), (4, 2563), (4, 4096), (8200, 64), (4099, 4096)])
def test_tanh_norm_forms(gpu, dtype, rows, width):
    rng = np.random.default_rng(width)
    x0 = rng.standard_normal((rows, width)) * 2
    y = rounded(rng.standard_normal((rows, width)) * .3, dtype)
    bias = rng.standard_normal(width)
    plain, norm = tanh_parts(rng, width)
    for b in (None, bias):
        x = dev(x0)
        h = ho.tanh_norm(x, norm, y=dev(y, dtype), bias=None if b is None else dev(b), dtype=dtype)
        want = x0 + y + (0.0 if b is None else b)
        close(x, want, 2e-6)
        close(h, ref.tanh_norm(want, *plain), tol(dtype, 2e-6, 5e-3))


def test_tanh_norm_of_tiny_and_of_huge_numbers(gpu):
    """Relative precision around zero, no overflow far out."""
    x0 = np.concatenate([np.geomspace(1e-7, 1e30, 500), -np.geomspace(1e-7, 1e30, 500), [0.0, 0.3, -0.3, 0.29999, 0.30001, 1e38, -1e38, 20.0]])[None]
    one, zero = torch.ones(x0.shape[1], device=gpu), torch.zeros(x0.shape[1], device=gpu)
    h = host(ho.tanh_norm(dev(x0), ho.TanhNorm(1.0, one, zero), y=torch.zeros(x0.shape, device=gpu), dtype=torch.float32))
    want = np.tanh(dev(x0).double().cpu().numpy())
    assert (np.abs(h - want) <= 1e-6 * np.abs(want)).all()


@pytest.mark.parametrize("rows", [1, 6, 64])
def test_tanh_norm_takes_the_pieces_of_a_product(gpu, rows):
    rng = np.random.default_rng(rows)
    width, bf = 512, torch.bfloat16
    y = ops.linear(dev(rng.standard_normal((rows, 4096)), bf), dev(rng.standard_normal((width, 4096)) * .02, bf), defer=True)
    assert isinstance(y, ops.SplitKSum)
    x0, bias, (plain, norm) = rng.standard_normal((rows, width)), rng.standard_normal(width), tanh_parts(rng, width)
    want = x0 + host(y.partial).sum(0) + bias
    x = dev(x0)
    h = ho.tanh_norm(x, norm, y=y, bias=dev(bias))
    close(x, want, 2e-6)
    close(h, ref.tanh_norm(want, *plain), 5e-3)


@BOTH
@pytest.mark.parametrize("width", [16, 77, 2048])
def test_embedding_behind_a_norm(gpu, dtype, width):
    rng = np.random.default_rng(width)
    embed = rounded(rng.standard_normal((11, width)), dtype)
    (first, first_norm), (plain, norm) = tanh_parts(rng, width), tanh_parts(rng, width)
    ids = torch.tensor([3, 0, 10, 10, 7], device=gpu)
    x = torch.full((5, width), float("nan"), device=gpu)
    h = ho.tanh_norm(x, norm, tokens=ids, embed=dev(embed, dtype), embed_scale=1.75, embed_norm=first_norm, dtype=dtype)
    want = ref.tanh_norm(embed[ids.cpu()] * 1.75, *first)
    close(x, want, 2e-6)
    close(h, ref.tanh_norm(want, *plain), tol(dtype, 2e-6, 5e-3))


@BOTH
@pytest.mark.parametrize("rows,cols", [(6, 8), (6, 30), (3, 352), (8200, 72), (64, 12288)])
@pytest.mark.parametrize("p,q", [(0.3, -0.8), (-4.0, 2.0)])
def test_xielu(gpu, dtype, rows, cols, p, q):
    rng = np.random.default_rng(cols)
    x, bias = rounded(rng.standard_normal((rows, cols)) * 3, dtype), rng.standard_normal(cols)
    x[0, :8] = 0.0
    bias[:8] = [0.0, -1e-6, 1e-6, -0.499, -0.501, -80.0, 30.0, -1e-3]
    got = ho.xielu(dev(x, dtype), dev(bias), ref.softplus(p), 0.5 + ref.softplus(q))
    want = ref.xielu(x + bias, p, q)
    close(got, want, tol(dtype, 1e-6, 4e-3))
    terms = np.abs(want[0, :8]) + np.abs(x + bias)[0, :8]           # which may cancel
    assert (np.abs(host(got)[0, :8] - want[0, :8]) <= tol(dtype, 1e-6, 5e-3) * terms).all()


@BOTH
def test_scaled_softcap(gpu, dtype):
    x = rounded(np.random.default_rng(0).standard_normal((3, 1031)) * 40, dtype)
    close(ho.softcap(dev(x, dtype), 7.5, 0.3), 7.5 * np.tanh(0.3 * x / 7.5), 1e-6)


# ------------------------------------------------------------------ pages
KEY_ORDER = np.array([8 * (r // 4) + 4 * x + r % 4 for x in range(2) for r in range(16)])      # of a tile's tokens, for keys


def to_pages(keys, values):
    """[blocks, kv_heads, block_size, entries] each, in tiles of 32 tokens as the kernels keep them."""
    b, h, bs, n = keys.shape
    k = keys.reshape(b, h, bs // 32, 32, n // 8, 8)[:, :, :, KEY_ORDER].transpose(0, 1, 2, 4, 3, 5)
    v = values.reshape(b, h, bs // 32, 4, 8, -1, 16).transpose(0, 1, 2, 5, 3, 6, 4)
    return k, v


def from_pages(keys, values):
    """The entries of every slot, [blocks * block_size, kv_heads, entries]."""
    b, h, tiles, groups = keys.shape[:4]
    k = keys[:, :, :, :, np.argsort(KEY_ORDER)].transpose(0, 2, 4, 1, 3, 5).reshape(b * tiles * 32, h, groups * 8)
    return k, values.transpose(0, 2, 4, 6, 1, 3, 5).reshape(b * tiles * 32, h, -1)


# ------------------------------------------------------------------ front end
@BOTH
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(6, 2, 24, 16), (3, 1, 10, 7), (16, 2, 128, 128), (32, 8, 64, 128), (8, 1, 64, 32), (2, 1, 200, 40),
                                                     (2, 2, 40, 200), (40, 8, 128, 96), (5, 5, 9, 300), (1, 1, 8, 8)])
@pytest.mark.parametrize("temp,norm_values", [((0.7, 32), True), ((0.5, 1), False), (None, True)])
@pytest.mark.parametrize("n", [9, 150])
def test_unit_head_front(gpu, dtype, heads, kv_heads, dim, vdim, temp, norm_values, n):
    rng = np.random.default_rng(heads * dim)
    bs, nblk, qx_rows, eps = 64, 4, 4, 1e-2
    s = ho.TalkShape(heads, kv_heads, dim, vdim, 1.0, eps, norm_values, *((temp[0], temp[1]) if temp else ()))
    off = [8, 8 + -(-heads * dim // 8) * 8]
    off.append(off[1] + -(-kv_heads * dim // 8) * 8)
    cols = -(-(off[2] + kv_heads * vdim + 5) // 8) * 8
    x = rounded(rng.standard_normal((n, cols)) * .2, dtype)
    pos = np.array([0, 30, 31, 32, 62, 63, 64, 1000, 70000])                                        # around where the factor changes
    slots = np.array([5, 31, 32, -1, 64, 95, 300, 0, 33], np.int32)                                  # one padding row, one outside the pool
    if n > 9:                                                    # runs of tokens that start and end inside of tiles and groups of eight
        runs = [np.arange(101, 134), np.arange(192, 256), np.arange(66, 77), np.arange(134, 167)]
        slots = np.concatenate([slots] + runs).astype(np.int32)
        assert len(slots) == n
        pos = np.concatenate([pos, rng.integers(0, 5000, n - 9)])
    shape = nblk, kv_heads, bs // 32
    keys = torch.full((*shape, s.key_pad // 8, 32, 8), 7.0, dtype=dtype, device=gpu)
    values = torch.full((*shape, s.vdim_pad // 16, 4, 16, 8), 7.0, dtype=dtype, device=gpu)
    qx = torch.full((qx_rows, heads, s.key_pad), float("nan"), dtype=dtype, device=gpu)
    proj = dev(x, dtype)
    ho.unit_head_front(s, proj, off, dev(pos, torch.int64), dev(slots, torch.int32), keys, values, qx, qx_rows)
    q = rms_norm(x[:, off[0]:off[0] + heads * dim].reshape(n, heads, dim), 1.0, eps)
    if temp:
        q = q * ref.query_temperature(pos, *temp)[:, None, None]
    k = rms_norm(x[:, off[1]:off[1] + kv_heads * dim].reshape(n, kv_heads, dim), 1.0, eps)
    v = x[:, off[2]:off[2] + kv_heads * vdim].reshape(n, kv_heads, vdim)
    if norm_values:
        v = rms_norm(v, 1.0, eps)
    t = tol(dtype, 2e-6, 5e-3)
    padded = np.zeros((qx_rows, heads, s.key_pad))
    padded[:, :, :dim] = q[:qx_rows]
    for r in range(qx_rows):                                     # row by row: the factor grows
        close(qx[r], padded[r], t)
    width = heads * dim
    for r in range(qx_rows, n):
        close(proj[r, off[0]:off[0] + width], q[r].ravel(), t)
    left = np.r_[0:off[0], off[0] + width:cols]
    assert np.array_equal(host(proj[:qx_rows]), x[:qx_rows]) and np.array_equal(host(proj)[:, left], x[:, left])
    for got, want, size in zip(from_pages(host(keys), host(values)), (k, v), (dim, vdim)):
        for i, slot in enumerate(slots):
            if 0 <= slot < nblk * bs:
                close(torch.tensor(got[slot, :, :size]), want[i], t)
                assert not got[slot, :, size:].any()
        assert (got[[i for i in range(nblk * bs) if i not in slots]] == 7.0).all()


# ------------------------------------------------------------------ attention
class Pages:
    """Random unit keys and values of several sequences in shuffled pages; every row that belongs to nobody is NaN."""

    def __init__(self, rng, lens, s, bs, dtype):
        self.k = [rounded(rms_norm(rng.standard_normal((n, s.kv_heads, s.dim)), 1.0, 0.0), dtype) for n in lens]
        self.v = [rounded(rms_norm(rng.standard_normal((n, s.kv_heads, s.vdim)), 1.0, 0.0), dtype) for n in lens]
        counts = [-(-n // bs) for n in lens]
        tables = np.full((len(lens), max(counts) + 1), -1, np.int32)
        ids, at = rng.permutation(sum(counts) + 2), 0
        keys = np.full((len(ids), s.kv_heads, bs, s.key_pad), np.nan)
        values = np.full((len(ids), s.kv_heads, bs, s.vdim_pad), np.nan)
        for i, n in enumerate(lens):
            for b in range(counts[i]):
                block = tables[i, b] = ids[at]
                at += 1
                m = min(bs, n - b * bs)
                for pages, data, size in ((keys, self.k[i], s.dim), (values, self.v[i], s.vdim)):
                    pages[block, :, :m] = 0.0
                    pages[block, :, :m, :size] = data[b * bs:b * bs + m].transpose(1, 0, 2)
        self.pages, self.tables = tuple(dev(p, dtype) for p in to_pages(keys, values)), dev(tables, torch.int32)


def one_query(s, talk, q, k, v):
    """``q`` [heads, dim] over the keys [n, kv_heads, dim]."""
    group, w = s.heads // s.kv_heads, []
    for h in range(s.heads):
        z = k[:, h // group] @ q[h] * s.scale
        top = max(z.max(), 0.0)
        p = np.exp(z - top)
        w.append(p / (p.sum() + np.exp(-top)))
    w = talk @ np.stack(w)
    return np.stack([w[h] @ v[:, h // group] for h in range(s.heads)]) * s.out_scale


def standing_out(rng, s, k, pos, dtype):
    """A query for whose heads the keys at the edges of what it sees stand out: the first, the last, and the one behind it."""
    q = rms_norm(rng.standard_normal((s.heads, s.dim)), 1.0, 0.0)
    for h, at in zip(range(s.heads), (0, pos, pos + 1, pos // 2)):
        if 0 <= at < len(k):
            q[h] = k[at, h // (s.heads // s.kv_heads)]
    return rounded(q * 4.0 / (s.scale * s.dim), dtype)           # such a key's score is 4


SHAPES = [(6, 2, 24, 16), (1, 1, 10, 7), (32, 4, 128, 128), (40, 2, 96, 32), (4, 2, 320, 300), (7, 7, 64, 64), (64, 8, 16, 24), (20, 1, 200, 160),
          (9, 3, 48, 120), (66, 3, 32, 32)]


def mixing(rng, heads, dtype):
    """No head keeps its own weights; signs differ."""
    return rounded(rng.standard_normal((heads, heads)) * heads ** -0.5, dtype)


@BOTH
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", SHAPES)
@pytest.mark.parametrize("scale", [0.3, 1e-3])
def test_talking_attention_rows(gpu, dtype, heads, kv_heads, dim, vdim, scale):
    rng = np.random.default_rng(dim)
    s = ho.TalkShape(heads, kv_heads, dim, vdim, scale, 0.0, out_scale=0.6)
    lens, bs = [1, 31, 33, 64, 130, 330], 32
    p = Pages(rng, lens, s, bs, dtype)
    ctx, row_seq = [1, 31, 2, 64, 129, 330, 32, 193, 65, 0], [0, 1, 2, 3, 4, 5, 4, 5, 4, 0]          # the last row is padding
    q = np.stack([standing_out(rng, s, p.k[i], max(c - 1, 0), dtype) for c, i in zip(ctx, row_seq)])
    talk = mixing(rng, heads, dtype)
    qx = np.zeros((len(ctx), heads, s.key_pad))
    qx[:, :, :dim] = q
    want = np.zeros((len(ctx), heads, vdim))
    for r, (c, i) in enumerate(zip(ctx, row_seq)):
        if c:
            want[r] = one_query(s, talk, q[r], p.k[i][:c], p.v[i][:c])
    for splits in (0, 1, 3):
        out = torch.full((len(ctx), heads * vdim + 4), 9.0, dtype=dtype, device=gpu)
        ho.talking_attention(s, dev(qx, dtype), *p.pages, dev(talk, dtype), p.tables, dev(ctx, torch.int32), out[:, :heads * vdim],
                             row_seq=dev(row_seq, torch.int32), splits=splits)
        for r in range(len(ctx)):
            close(out[r, :heads * vdim], want[r].ravel(), tol(dtype, 1e-5, 2e-2))
        assert (out[:, heads * vdim:] == 9.0).all()


@BOTH
@pytest.mark.parametrize("size", [200.0, -200.0, 60.0, -12.0])
def test_scores_beyond_what_exponentials_hold_and_below_the_sink(gpu, dtype, size):
    """All scores far above zero: the sink is nothing.  Far below: everything is the sink's, but for what is left."""
    rng = np.random.default_rng(3)
    s = ho.TalkShape(4, 2, 32, 32, 0.5, 0.0)
    n = 100
    p = Pages(rng, [n], s, 32, dtype)
    key = np.abs(rng.standard_normal(32))
    k = rounded(np.broadcast_to(key, (n, 2, 32)) + 0.01 * rng.standard_normal((n, 2, 32)), dtype)
    p.pages[0].zero_()
    for b in range(4):
        m = min(32, n - 32 * b)
        tile = np.zeros((1, 2, 32, 32))
        tile[0, :, :m] = k[32 * b:32 * b + m].transpose(1, 0, 2)
        p.pages[0][p.tables[0, b]] = dev(to_pages(tile, tile)[0][0], dtype)
    q = rounded(np.broadcast_to(key * size / (0.5 * key @ key), (1, 4, 32)), dtype)
    talk = mixing(rng, 4, dtype)
    want = one_query(s, talk, q[0], k, p.v[0])
    out = torch.empty((1, 128), dtype=dtype, device=gpu)
    ho.talking_attention(s, dev(q, dtype), *p.pages, dev(talk, dtype), p.tables, dev([n], torch.int32), out)
    if size == -200.0:
        assert (out.abs() <= 1e-30).all()
    else:
        close(out, want.reshape(1, -1), tol(dtype, 2e-5, 2e-2))
    if dtype == torch.bfloat16 and size != -200.0:
        out = torch.empty((n, 128), dtype=dtype, device=gpu)
        rows = np.broadcast_to(q.reshape(1, -1), (n, 128))
        cu = dev([0, n], torch.int32)
        ho.talking_prefill(s, dev(rows, dtype), *p.pages, dev(talk, dtype), p.tables, dev([0], torch.int32), cu, cu, n, n, out)
        for t in (0, 1, 31, 32, 99):
            close(out[t], one_query(s, talk, q[0], k[:t + 1], p.v[0][:t + 1]).ravel(), 2e-2)


def test_a_weight_of_one_head_moves_the_others(gpu):
    """The weights of head 1 alone, in the rows of the others."""
    rng, dtype = np.random.default_rng(8), torch.float32
    s = ho.TalkShape(3, 3, 8, 8, 1.0, 0.0)
    p = Pages(rng, [40], s, 32, dtype)
    q = rng.standard_normal((1, 3, 8))
    talk = np.zeros((3, 3))
    talk[:, 1] = [1.0, 0.5, -2.0]
    z = np.exp(p.k[0][:, 1] @ q[0, 1])
    w = z / (1 + z.sum())
    want = np.stack([talk[h, 1] * w @ p.v[0][:, h] for h in range(3)])
    qx = np.zeros((1, 3, 32))
    qx[:, :, :8] = q
    out = torch.empty((1, 24), device=gpu)
    ho.talking_attention(s, dev(qx), *p.pages, dev(talk), p.tables, dev([40], torch.int32), out)
    close(out, want.reshape(1, -1), 1e-5)


@BOTH
def test_rows_run_in_turns_when_their_scores_are_many(gpu, dtype, monkeypatch):
    rng = np.random.default_rng(4)
    s = ho.TalkShape(4, 2, 32, 32, 0.2, 0.0)
    lens = [70, 33, 96, 5, 61]
    p = Pages(rng, lens, s, 32, dtype)
    qx, talk, ctx = dev(rng.standard_normal((5, 4, 32)), dtype), dev(mixing(rng, 4, dtype), dtype), dev(lens, torch.int32)
    outs = []
    for limit in (1 << 28, 4 * 96 * 2, 1):
        monkeypatch.setattr(ho, "TALK_SCORES", limit)
        for row_seq in (None, torch.arange(5, dtype=torch.int32, device=gpu)):
            out = torch.empty((5, 128), dtype=dtype, device=gpu)
            ho.talking_attention(s, qx, *p.pages, talk, p.tables, ctx, out, row_seq=row_seq, max_keys=96, splits=1)
            outs.append(out)
    assert all(torch.equal(o, outs[0]) for o in outs)


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(6, 2, 24, 16), (6, 6, 64, 64), (1, 1, 8, 8), (8, 4, 128, 128), (16, 8, 128, 128), (11, 11, 72, 40),
                                                     (12, 3, 64, 128), (16, 4, 128, 64), (32, 8, 128, 128), (20, 20, 48, 56), (24, 2, 128, 96),
                                                     (30, 10, 64, 64), (32, 32, 128, 128), (17, 1, 128, 128)])
@pytest.mark.parametrize("bs", [32, 96])
@pytest.mark.parametrize("bounded", [True, False])
def test_talking_prefill(gpu, heads, kv_heads, dim, vdim, bs, bounded):
    """Portions behind a cached prefix; keys at the edges of what a query sees stand out, rows nobody sees are NaN."""
    rng, bf = np.random.default_rng(dim + heads), torch.bfloat16
    s = ho.TalkShape(heads, kv_heads, dim, vdim, 0.2, 0.0, out_scale=0.6)
    assert ho.talking_prefill_supported(s)
    lens, new = [130, 250, 64, 333], [130, 77, 64, 200]
    p = Pages(rng, lens, s, bs, bf)
    seqs = [2, 0, 3, 1]
    cu_q, cu_k = np.cumsum([0] + [new[i] for i in seqs]), np.cumsum([0] + [lens[i] for i in seqs])
    q = np.concatenate([np.stack([standing_out(rng, s, p.k[i], lens[i] - new[i] + t, bf) for t in range(new[i])]) for i in seqs])
    total = int(cu_q[-1])
    proj = torch.zeros((total, 8 + -(-heads * dim // 8) * 8), dtype=bf, device=gpu)
    proj[:, 8:8 + heads * dim] = dev(q.reshape(total, -1), bf)
    talk = mixing(rng, heads, bf)
    wide = torch.full((total, heads * vdim + 8), 9.0, dtype=bf, device=gpu)
    out = wide[:, :heads * vdim]
    ho.talking_prefill(s, proj[:, 8:], *p.pages, dev(talk, bf), p.tables, dev(seqs, torch.int32), dev(cu_q, torch.int32), dev(cu_k, torch.int32),
                       max(new), max(lens), out, max_score=20.0 if bounded else None)
    assert (wide[:, heads * vdim:] == 9.0).all()
    for j, i in enumerate(seqs):
        for t in range(0, new[i], 1 if heads <= 12 else 3):
            r, seen = int(cu_q[j]) + t, lens[i] - new[i] + t + 1
            close(out[r], one_query(s, talk, q[r], p.k[i][:seen], p.v[i][:seen]).ravel(), 2e-2)


@pytest.mark.parametrize("heads,lens", [(8, [70, 64, 200, 33, 96, 5, 61, 300, 129]), (12, [70, 64, 200, 33, 96, 5, 61, 300]), (6, [700] * 40), (16, [470] * 24),
                                        (14, [500] * 17), (32, [100] * 8), (8, [1100]), (10, [650, 40, 330]), (16, [900, 40]), (32, [1030])])
def test_prefill_and_rows_agree(gpu, heads, lens):
    """Eight sequences take another order of workgroups; many workgroups have more queries each; few queries of many keys are
    split over workgroups, of which short sequences leave some without keys."""
    rng, bf = np.random.default_rng(5), torch.bfloat16
    s = ho.TalkShape(heads, 2, 64, 64, 0.1, 0.0)
    p = Pages(rng, lens, s, 32, bf)
    cu = np.cumsum([0] + lens)
    q = dev(rms_norm(rng.standard_normal((cu[-1], heads, 64)), 1.0, 0.0), bf)
    talk = dev(mixing(rng, heads, bf), bf)
    a, b = (torch.empty((int(cu[-1]), heads * 64), dtype=bf, device=gpu) for _ in range(2))
    ho.talking_prefill(s, q.view(-1, heads * 64), *p.pages, talk, p.tables, torch.arange(len(lens), dtype=torch.int32, device=gpu), dev(cu, torch.int32),
                       dev(cu, torch.int32), max(lens), max(lens), a, max_score=s.max_score(max(lens)))
    ctx = np.concatenate([np.arange(1, n + 1) for n in lens])
    row_seq = np.repeat(np.arange(len(lens)), lens)
    ho.talking_attention(s, q, *p.pages, talk, p.tables, dev(ctx, torch.int32), b, row_seq=dev(row_seq, torch.int32), max_keys=max(lens))
    close(a, host(b), 1.5e-2)


def test_what_the_prompt_kernels_do_not_serve(gpu):
    for heads, dim, vdim in ((33, 64, 64), (8, 136, 64), (8, 64, 136), (8, 20, 64), (8, 64, 12)):
        assert not ho.talking_prefill_supported(ho.TalkShape(heads, heads, dim, vdim, 1.0, 0.0))


def test_a_bound_of_the_scores():
    s = ho.TalkShape(2, 2, 16, 16, 0.5, 0.0, True, 3.0, 40)
    assert s.max_score(39) == pytest.approx(1.05 * 8.0) and s.max_score(40) == pytest.approx(1.05 * 8.0 * (1 + 3 * np.log(2)))
    assert ho.TalkShape(2, 2, 16, 16, 0.5, 0.0).max_score(10 ** 6) == pytest.approx(1.05 * 8.0)
