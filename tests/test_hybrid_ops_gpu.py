"""The kernels of latent attention, the gated delta rule and the float32 residual stream, each alone, against
``oracle/merilorn_ref.py`` (float64) on random inputs made so that a wrong key, token or state shows."""
import numpy as np
import pytest
import torch

from infer_amd import hybrid_ops as ho, ops
from infer_amd.layers import yarn_rotary_table
from infer_amd.step_plan import CHUNK
from oracle import merilorn_ref as ref

pytestmark = pytest.mark.gpu
BOTH = pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["f32", "bf16"])


def tol(dtype, f32=2e-5, bf16=2e-2):
    return f32 if dtype == torch.float32 else bf16


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.array(a)).to("cuda").to(dtype).contiguous()


def rounded(a, dtype):
    """The values the kernel sees, as float64."""
    return torch.as_tensor(np.asarray(a, np.float64)).to(dtype).double().numpy()


def host(t):
    return t.detach().double().cpu().numpy()


def close(got, want, atol):
    got, want = host(got), np.asarray(want)
    assert np.isfinite(got).all()
    err = np.abs(got - want).max() / max(np.abs(want).max(), 1e-30)
    assert err <= atol, err


# ------------------------------------------------------------------ residual stream
@BOTH
@pytest.mark.parametrize("width", [8, 72, 129, 1000, 1024, 2563, 4096, 9000])
def test_residual_norm_forms(gpu, dtype, width):
    rng = np.random.default_rng(width)
    n, eps = 5, 1e-3
    x0, y = rng.standard_normal((n, width)), rounded(rng.standard_normal((n, width)) * 3, dtype)
    wp, wn = 1 + rng.standard_normal((2, width)) * .3
    embed = rounded(rng.standard_normal((11, width)), dtype)
    x = dev(x0)
    h = ho.residual_norm(x, eps, y=dev(y, dtype), w_post=dev(wp), w_pre=dev(wn), dtype=dtype)
    want = x0 + ref.rms_norm(y, wp, eps)
    close(x, want, 1e-6)
    close(h, ref.rms_norm(want, wn, eps), tol(dtype, 2e-6, 8e-3))
    x = torch.full((n, width), float("nan"), device="cuda")
    ids = torch.tensor([3, 0, 10, 10, 7], device="cuda")
    h = ho.residual_norm(x, eps, tokens=ids, embed=dev(embed, dtype), embed_scale=5.5, w_pre=dev(wn), dtype=dtype)
    close(x, embed[ids.cpu()] * 5.5, 1e-6)
    close(h, ref.rms_norm(embed[ids.cpu()] * 5.5, wn, eps), tol(dtype, 2e-6, 8e-3))
    x = dev(x0)
    assert ho.residual_norm(x, eps, y=dev(y, dtype), w_post=dev(wp), dtype=dtype) is None
    close(x, want, 1e-6)


def test_residual_norm_of_split_k_pieces(gpu):
    rng = np.random.default_rng(0)
    m, n, k = 7, 512, 4096
    a, w = dev(rng.standard_normal((m, k)), torch.bfloat16), dev(rng.standard_normal((n, k)) * .02, torch.bfloat16)
    y = ops.linear(a, w, defer=True)
    assert isinstance(y, ops.SplitKSum)
    x, wp = dev(rng.standard_normal((m, n))), 1 + rng.standard_normal(n) * .2
    want = host(x) + ref.rms_norm(host(a) @ host(w).T, wp, 1e-6)
    ho.residual_norm(x, 1e-6, y=y, w_post=dev(wp), dtype=torch.bfloat16)
    close(x, want, 1e-5)


@BOTH
@pytest.mark.parametrize("d", [8, 30, 352])
def test_gelu_tanh_and_mul(gpu, dtype, d):
    x = rounded(np.random.default_rng(d).standard_normal((6, 2 * d)) * 4, dtype)
    x[0, 0], x[1, 0] = 60.0, -60.0
    close(ho.gelu_tanh_and_mul(dev(x, dtype)), ref.gelu_tanh(x[:, :d]) * x[:, d:], tol(dtype, 1e-6, 8e-3))


# ------------------------------------------------------------------ latent attention: front end and products
@BOTH
@pytest.mark.parametrize("heads,dim,rot,rot_dims,rank", [(3, 16, 8, 8, 40), (5, 20, 12, 8, 33), (2, 64, 64, 64, 128), (1, 6, 2, 2, 3)])
def test_latent_front(gpu, dtype, heads, dim, rot, rot_dims, rank):
    rng = np.random.default_rng(rank)
    n, eps, qx_rows = 6, 1e-4, 4
    rank_pad = -(-rank // 32) * 32
    row = rank_pad + -(-rot // 32) * 32
    qn = heads * (dim + rot)
    kv_off = -(-qn // 8) * 8
    cols = kv_off + rank + rot + 3
    p0 = rounded(rng.standard_normal((n, cols)), dtype)
    norm = 1 + rng.standard_normal(rank) * .3
    pos = np.array([0, 1, 17, 300, 511, 64])
    slots = np.array([5, 70, -1, 0, 127, 64])
    scaling = dict(factor=4.0, original=128, fast=8.0, slow=1.0)
    table = yarn_rotary_table(rot_dims, 512, 1000.0, scaling, "cuda")
    freq, mag = ref.yarn_frequencies(rot_dims, 1000.0, scaling)
    proj = dev(p0, dtype)
    cache = torch.full((2, 64, row), 77.0, dtype=dtype, device="cuda")
    qx = torch.full((qx_rows, heads, row), 55.0, dtype=dtype, device="cuda")
    ho.latent_front(proj, heads, dim, rot, rot_dims, kv_off, rank, dev(norm), eps, table, dev(pos, torch.int64),
                    dev(slots, torch.int32), cache, rank_pad, qx, qx_rows)
    c = ref.rms_norm(p0[:, kv_off:kv_off + rank], norm, eps)
    kr = ref.rotate_interleaved(p0[:, kv_off + rank:kv_off + rank + rot], pos, freq, mag)
    want = np.full((128, row), 77.0)
    for t, s in enumerate(slots):
        if s >= 0:
            want[s] = 0
            want[s, :rank], want[s, rank_pad:rank_pad + rot] = c[t], kr[t]
    assert np.abs(host(cache).reshape(128, row) - want).max() <= tol(dtype, 1e-5, 3e-2)
    assert (host(cache).reshape(128, row)[want == 0] == 0).all()
    q = p0[:, :qn].reshape(n, heads, dim + rot)
    qr = ref.rotate_interleaved(q[..., dim:], pos, freq, mag)
    got = host(qx)
    assert (got[..., :rank_pad] == 55).all() and (got[..., rank_pad + rot:] == 0).all()
    close(qx[..., rank_pad:rank_pad + rot], qr[:qx_rows], tol(dtype, 1e-5))
    after = host(proj)
    assert np.array_equal(after[:qx_rows], p0[:qx_rows]) and np.array_equal(after[:, qn:], p0[:, qn:])
    rest = after[qx_rows:, :qn].reshape(n - qx_rows, heads, dim + rot)
    assert np.array_equal(rest[..., :dim], q[qx_rows:, :, :dim])
    assert np.abs(rest[..., dim:] - qr[qx_rows:]).max() <= tol(dtype, 1e-5, 3e-2)


@BOTH
@pytest.mark.parametrize("m,heads,n,k,lead", [(1, 3, 40, 16, 8), (5, 2, 24, 48, 0), (70, 5, 33, 20, 3), (200, 2, 128, 96, 8), (17, 1, 7, 5, 0)])
def test_head_matmul(gpu, dtype, m, heads, n, k, lead):
    rng = np.random.default_rng(m)
    x = rounded(rng.standard_normal((m, heads, k + lead)), dtype)
    w = rounded(rng.standard_normal((heads, n, k)), dtype)
    g = rounded(rng.standard_normal((m, heads)), dtype)
    wp = np.zeros((heads, -(-n // 16) * 16, -(-k // 32) * 32))
    wp[:, :n, :k] = w
    out = torch.full((m, heads, n + lead), 9.0, dtype=dtype, device="cuda")
    want = np.einsum("mhk,hnk->mhn", x[..., :k], w)
    ho.head_matmul(dev(x, dtype)[..., :k], dev(wp, dtype), out, n, k, gate=dev(g, dtype))
    close(out[..., :n], want * ref.sigmoid(g)[..., None], tol(dtype, 1e-5, 1e-2))
    assert (host(out)[..., n:] == 9).all()
    ho.head_matmul(dev(x, dtype)[..., :k], dev(wp, dtype), out, n, k)
    close(out[..., :n], want, tol(dtype, 1e-5, 1e-2))


# ------------------------------------------------------------------ latent attention: rows
def latent_case(rng, ctx, heads, row, rank_pad, bs, dtype, spare=3):
    """Sequences of the given lengths in shuffled blocks of a pool whose unused rows are NaN."""
    need = [-(-c // bs) for c in ctx]
    nblk = sum(need) + spare
    ids = rng.permutation(nblk)
    tables = np.full((len(ctx), max(max(need), 1) + 1), -1)
    cache = np.full((nblk, bs, row), np.nan)
    keys = []
    for s, c in enumerate(ctx):
        tables[s, :need[s]] = ids[sum(need[:s]):sum(need[:s + 1])]
        k = rounded(rng.standard_normal((c, row)), dtype)
        keys.append(k)
        for t in range(c):
            cache[tables[s, t // bs], t % bs] = k[t]
    q = rounded(rng.standard_normal((len(ctx), heads, row)), dtype)
    return q, keys, cache, tables


def latent_want(q, k, rank_pad, scale):
    s = q @ k.T * scale
    p = np.exp(s - s.max(-1, keepdims=True))
    return p / p.sum(-1, keepdims=True) @ k[:, :rank_pad]


SIZES = [(3, 96, 64), (7, 160, 96), (17, 192, 128), (2, 64, 32), (16, 320, 256), (40, 576, 512), (5, 160, 128), (3, 800, 768)]


@BOTH
@pytest.mark.parametrize("heads,row,rank_pad", SIZES)
@pytest.mark.parametrize("splits", [0, 1, 3, 16])
def test_latent_attention_lengths_around_tiles_and_blocks(gpu, dtype, heads, row, rank_pad, splits):
    rng = np.random.default_rng(row)
    bs, scale = 64, row ** -0.5
    ctx = [1, 2, 31, 32, 33, 63, 64, 65, 127, 128, 129, 500]
    q, keys, cache, tables = latent_case(rng, ctx, heads, row, rank_pad, bs, dtype)
    out = ho.latent_attention(dev(q, dtype), dev(cache, dtype), dev(tables, torch.int32), dev(ctx, torch.int32), scale, rank_pad,
                              splits=splits)
    for s, k in enumerate(keys):
        close(out[s], latent_want(q[s], k, rank_pad, scale), tol(dtype))


@BOTH
@pytest.mark.parametrize("splits", [1, 4])
@pytest.mark.parametrize("at", [0, 31, 32, 63, 64, 100, 191, 192, 316, 317])
def test_latent_attention_one_key_stands_out(gpu, dtype, splits, at):
    """The query is aimed at one key; the last visible one and the first invisible one are told apart."""
    rng = np.random.default_rng(at)
    heads, row, rank_pad, n = 5, 160, 128, 318
    q, keys, cache, tables = latent_case(rng, [n], heads, row, rank_pad, 32, dtype)
    aim = np.broadcast_to(keys[0][at] * 2.0, (4, heads, row))
    ctx = [at + 1, max(at, 1), n, min(at + 2, n)]
    out = ho.latent_attention(dev(aim, dtype), dev(cache, dtype), dev(tables, torch.int32), dev(ctx, torch.int32), 1.0, rank_pad,
                              row_seq=dev([0] * 4, torch.int32), splits=splits)
    for r, c in enumerate(ctx):
        close(out[r], latent_want(aim[r], keys[0][:c], rank_pad, 1.0), tol(dtype))
        hit = np.abs(host(out[r, 0]) - keys[0][at, :rank_pad]).max() < 0.05
        assert hit == (c > at)


@BOTH
def test_latent_attention_rows_of_one_sequence_and_empty_rows(gpu, dtype):
    rng = np.random.default_rng(5)
    q, keys, cache, tables = latent_case(rng, [100, 40], 4, 96, 64, 32, dtype)
    seq, ctx = [0, 0, 1, 0, 1, 1], [3, 99, 40, 100, 1, 0]
    qq = rounded(rng.standard_normal((6, 4, 96)), dtype)
    for splits in (1, 2):
        out = ho.latent_attention(dev(qq, dtype), dev(cache, dtype), dev(tables, torch.int32), dev(ctx, torch.int32), 0.1, 64,
                                  row_seq=dev(seq, torch.int32), splits=splits)
        for r in range(5):
            close(out[r], latent_want(qq[r], keys[seq[r]][:ctx[r]], 64, 0.1), tol(dtype))
        assert (host(out[5]) == 0).all()


def test_latent_gather(gpu):
    rng = np.random.default_rng(6)
    q, keys, cache, tables = latent_case(rng, [70, 1, 33], 1, 96, 64, 32, torch.bfloat16)
    out = ho.latent_gather(dev(cache, torch.bfloat16), dev(tables, torch.int32), dev([2, 0], torch.int32), dev([0, 33, 103], torch.int32), 103, 70)
    assert np.array_equal(host(out), np.concatenate([keys[2], keys[0]]))


@pytest.mark.parametrize("heads,dim,rot,vdim", [(3, 16, 8, 24), (5, 48, 16, 40), (2, 96, 32, 64), (2, 64, 32, 128), (3, 128, 64, 128), (1, 192, 64, 104), (2, 24, 40, 8)])
def test_latent_prefill(gpu, heads, dim, rot, vdim):
    """Portions with and without a prefix, lengths around the tiles; one query-key pair stands out."""
    rng = np.random.default_rng(dim)
    bf = torch.bfloat16
    sq, sk = [64, 1, 130, 200, 33], [64, 40, 130, 257, 97]
    cu_q, cu_k = np.concatenate(([0], np.cumsum(sq))), np.concatenate(([0], np.cumsum(sk)))
    q = rounded(rng.standard_normal((cu_q[-1], heads * (dim + rot))), bf)
    kp, kr = rounded(rng.standard_normal((cu_k[-1], heads * dim)), bf), rounded(rng.standard_normal((cu_k[-1], rot)), bf)
    v, g = rounded(rng.standard_normal((cu_k[-1], heads * vdim)), bf), rounded(rng.standard_normal((cu_q[-1], heads)), bf)
    for s, i, j in ((3, 199, 0), (3, 150, 32), (2, 129, 129), (4, 32, 96), (2, 64, 63)):
        for h in range(heads):      # q_i = 3 k_j
            q[cu_q[s] + i, h * (dim + rot):(h + 1) * (dim + rot)] = rounded(
                3 * np.concatenate([kp[cu_k[s] + j, h * dim:(h + 1) * dim], kr[cu_k[s] + j]]), bf)
    scale = 1.5 * (dim + rot) ** -0.5
    out = torch.full((int(cu_q[-1]), heads * vdim), float("nan"), dtype=bf, device="cuda")
    ho.latent_prefill(dev(q, bf), dev(kp, bf), dev(kr, bf), dev(v, bf), dev(g, bf), out, dev(cu_q, torch.int32),
                      dev(cu_k, torch.int32), max(sq), heads, dim, rot, vdim, scale)
    for s in range(len(sq)):
        a, b = slice(cu_q[s], cu_q[s + 1]), slice(cu_k[s], cu_k[s + 1])
        qs = q[a].reshape(sq[s], heads, dim + rot)
        ks = np.concatenate([kp[b].reshape(sk[s], heads, dim), np.broadcast_to(kr[b][:, None], (sk[s], heads, rot))], -1)
        vs = v[b].reshape(sk[s], heads, vdim)
        sc = np.einsum("ihd,jhd->hij", qs, ks) * scale
        sc = np.where(np.arange(sk[s])[None] <= np.arange(sq[s])[:, None] + sk[s] - sq[s], sc, -np.inf)
        p = np.exp(sc - sc.max(-1, keepdims=True))
        o = np.einsum("hij,jhd->ihd", p / p.sum(-1, keepdims=True), vs) * ref.sigmoid(g[a])[..., None]
        close(out[a], o.reshape(sq[s], -1), 2e-2)


# ------------------------------------------------------------------ gated delta rule
class DeltaCase:
    def __init__(self, heads, kv_heads, dim, vdim, taps, n, dtype, seed=0, decay=-2.0, slots=3):
        rng = np.random.default_rng(seed)
        self.s = s = ho.DeltaShape(heads, kv_heads, dim, vdim, taps, 1e-4)
        self.dtype, self.n = dtype, n
        self.beta_off = -(-s.channels // 8) * 8
        self.proj = rounded(rng.standard_normal((n, self.beta_off + heads + 5)), dtype)
        self.decay = rounded(rng.standard_normal((n, heads * dim)), dtype)
        self.gate = rounded(rng.standard_normal((n, heads * vdim)), dtype)
        self.conv = rng.standard_normal((s.channels, taps)) * .7
        self.a_log, self.dt = rng.standard_normal(heads), rng.standard_normal(heads * dim) + decay
        self.norm = 1 + .3 * rng.standard_normal(vdim)
        # whatever is in the slots before a sequence starts must not matter
        self.state = torch.full((slots, heads, s.state_rows, s.state_cols), float("nan"), device="cuda")
        self.ring = torch.full((slots, taps, s.channels), float("nan"), dtype=dtype, device="cuda")

    @property
    def weights(self):
        return [dev(x) for x in (self.conv, self.a_log, self.dt, self.norm)]

    def want(self):
        s, n = self.s, self.n
        qkv = ref.silu(ref.causal_conv(self.proj[:, :s.channels], self.conv))
        qk = s.kv_heads * s.dim
        q = ref.unit_norm(qkv[:, :qk].reshape(n, s.kv_heads, s.dim)) * s.dim ** -0.5
        k = ref.unit_norm(qkv[:, qk:2 * qk].reshape(n, s.kv_heads, s.dim))
        v = qkv[:, 2 * qk:].reshape(n, s.heads, s.vdim)
        beta = ref.sigmoid(self.proj[:, self.beta_off:self.beta_off + s.heads])
        g = -np.exp(self.a_log)[:, None] * ref.softplus(self.decay + self.dt).reshape(n, s.heads, s.dim)
        o, states = np.zeros((n, s.heads, s.vdim)), []
        for h in range(s.heads):
            j = h // (s.heads // s.kv_heads)
            o[:, h], st = ref.delta_scan(q[:, j], k[:, j], v[:, h], g[:, h], beta[:, h])
            states.append(st)
        o = ref.rms_norm(o, self.norm, s.eps) * ref.sigmoid(self.gate).reshape(n, s.heads, s.vdim)
        return o.reshape(n, -1), np.stack(states)

    def run(self, cuts, slot=1):
        """The tokens in portions of the given sizes; portions of one token take the decode kernel."""
        s, lo, outs = self.s, 0, []
        for c in cuts:
            a = [dev(x[lo:lo + c], self.dtype) for x in (self.proj, self.decay, self.gate)]
            out = torch.full((c, s.heads * s.vdim), float("nan"), dtype=self.dtype, device="cuda")
            pos = dev(np.arange(lo, lo + c), torch.int64)
            if c == 1:
                ho.delta_step(s, a[0], self.beta_off, a[1], a[2], *self.weights, self.ring, self.state, dev([slot], torch.int32), pos, out)
            else:
                chunks = [(r, min(CHUNK, c - r), lo + r, lo, slot, 0) for r in range(0, c, CHUNK)]
                ring = [(slot, c - 1 - r) for r in range(c)]
                ho.delta_chunks(s, a[0], self.beta_off, a[1], a[2], *self.weights, self.ring, self.state,
                                dev([(0, len(chunks), slot, lo)], torch.int32), dev(chunks, torch.int32), dev(ring, torch.int32), pos, 0, out)
            outs.append(out)
            lo += c
        assert lo == self.n
        return torch.cat(outs), self.state[slot]

    def check(self, cuts, slot=1):
        out, state = self.run(cuts, slot)
        want, want_state = self.want()
        close(out, want, tol(self.dtype, 3e-5, 1e-2))
        close(state[:, :self.s.dim, :self.s.vdim], want_state, 3e-5)      # float32 in both types
        rest = host(state)
        assert (rest[:, self.s.dim:] == 0).all() and (rest[:, :, self.s.vdim:] == 0).all()


DELTA_SIZES = [(3, 3, 48, 32, 4), (4, 2, 24, 16, 4), (3, 1, 16, 40, 3), (2, 1, 128, 128, 4), (1, 1, 100, 20, 2), (2, 2, 5, 7, 1),
               (2, 1, 192, 64, 5), (1, 1, 256, 256, 4), (1, 1, 40, 300, 4)]


@BOTH
@pytest.mark.parametrize("size", DELTA_SIZES)
def test_delta_whole_prompt_then_tokens(gpu, dtype, size):
    DeltaCase(*size, 45, dtype).check([37] + [1] * 8)


@pytest.mark.parametrize("size", DELTA_SIZES[:4])
@pytest.mark.parametrize("cuts", [[50], [1] * 50, [2] * 25, [16, 17, 15, 2], [3, 2, 1, 1, 33, 1, 9], [1, 2, 3, 4, 5, 6, 7, 8, 9, 5]])
def test_delta_any_cut(gpu, size, cuts):
    DeltaCase(*size, 50, torch.float32, seed=1).check(cuts)


@pytest.mark.parametrize("decay", [-9.0, 0.0, 5.0, 40.0])
def test_delta_decay_strengths(gpu, decay):
    """From almost none to a state that is gone after one token: nothing overflows, nothing is lost."""
    DeltaCase(2, 1, 48, 64, 4, 70, torch.float32, seed=2, decay=decay).check([64, 1, 5])


def test_delta_first_token_is_still_read_far_later(gpu):
    """Token 0 alone writes; almost no decay; the last query asks for what it wrote."""
    c = DeltaCase(1, 1, 32, 32, 1, 300, torch.float32, seed=3, decay=-16.0)
    c.proj[1:, c.beta_off] = -60.0                    # write strength 0 behind token 0
    c.proj[299, :32] = c.proj[0, 32:64]               # the query of the last token is the key of the first
    c.conv[:64] = 1.0
    c.check([1, 280] + [1] * 19)
    want, _ = c.want()
    c2 = DeltaCase(1, 1, 32, 32, 1, 300, torch.float32, seed=3, decay=-16.0)
    assert np.abs(want[299] - c2.want()[0][299]).max() > 0.1


def test_delta_batches_slots_and_padding(gpu):
    """Several sequences in one call, each in its slot; padding rows touch nothing; a slot is used again."""
    cases = [DeltaCase(4, 2, 24, 16, 4, 33 + i, torch.float32, seed=10 + i) for i in range(3)]
    for c in cases[1:]:
        c.conv, c.a_log, c.dt, c.norm = cases[0].conv, cases[0].a_log, cases[0].dt, cases[0].norm
    c0, s = cases[0], cases[0].s
    slots = [2, 0, 1]
    n = [31, 32, 17]
    cat = lambda name: dev(np.concatenate([getattr(c, name)[:k] for c, k in zip(cases, n)]), torch.float32)
    chunks, portions, ring, pos, row = [], [], [], [], 0
    for slot, k in zip(slots, n):
        portions.append((len(chunks), -(-k // 16), slot, 0))
        chunks += [(row + r, min(16, k - r), r, 0, slot, 0) for r in range(0, k, 16)]
        ring += [(slot, k - 1 - r) for r in range(k)]
        pos += range(k)
        row += k
    out = torch.empty((row, s.heads * s.vdim), device="cuda")
    ho.delta_chunks(s, cat("proj"), c0.beta_off, cat("decay"), cat("gate"), *c0.weights, c0.ring, c0.state, dev(portions, torch.int32),
                    dev(chunks, torch.int32), dev(ring, torch.int32), dev(pos, torch.int64), 0, out)
    done = [host(out[sum(n[:i]):sum(n[:i + 1])]) for i in range(3)]
    for t in range(3):                                # three tokens of sequences 0 and 1 and a padding row
        rows = [cases[0], cases[1], cases[2]]
        step = lambda name: dev(np.stack([getattr(c, name)[min(k + t, c.n - 1)] for c, k in zip(rows, n)]), torch.float32)
        before = c0.state[1].clone()
        o = torch.full((3, s.heads * s.vdim), 5.0, device="cuda")
        active = [k + t < c.n for c, k in zip(cases, n)][:2]
        sl = [slots[i] if i < 2 and active[i] else -1 for i in range(3)]
        ho.delta_step(s, step("proj"), c0.beta_off, step("decay"), step("gate"), *c0.weights, c0.ring, c0.state, dev(sl, torch.int32),
                      dev([k + t for k in n], torch.int64), o)
        assert torch.equal(before, c0.state[1]) and (o[2] == 0).all()
        for i in range(2):
            if active[i]:
                done[i] = np.concatenate([done[i], host(o[i:i + 1])])
    for i in range(3):
        want = cases[i].want()[0][:len(done[i])]
        assert np.abs(done[i] - want).max() <= 3e-5 * np.abs(want).max()
    again = DeltaCase(4, 2, 24, 16, 4, 20, torch.float32, seed=20)
    again.state, again.ring = c0.state, c0.ring
    again.check([2, 1, 17], slot=2)


def test_sizes_outside_are_refused_on_the_host(gpu):
    with pytest.raises(RuntimeError):
        ho.delta_layout(300, 16)
    q = torch.zeros((1, 1, 40), dtype=torch.float32, device="cuda")
    with pytest.raises(RuntimeError):
        ho.latent_attention(q, torch.zeros((1, 32, 40), device="cuda"), torch.zeros((1, 1), dtype=torch.int32, device="cuda"),
                            torch.ones(1, dtype=torch.int32, device="cuda"), 1.0, 32)
