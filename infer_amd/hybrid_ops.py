"""Python entry points of the hybrid-model kernels (latent, grouped, masked and talking-heads attention, gated delta rule, linear
attention with a constant decay, selective state space, mixture of experts, float32 residual stream), beside ``ops``: shape and type
checks on the host, then one call into ``libinfer_kv.so`` on torch's current stream.  Activations are bfloat16 or float32; there is no CPU path."""
from __future__ import annotations

import ctypes
import math
from dataclasses import dataclass
from functools import lru_cache

import torch

from . import _lib
from .ops import SplitKSum, _require_gpu, _stream_ptr

ELEM = {torch.bfloat16: 0, torch.float32: 1}


def _ptr(t):
    return None if t is None else t.data_ptr()


def _rows(t: torch.Tensor, cols: int) -> int:
    """Row stride of a 2-D view with contiguous rows of at least ``cols`` elements."""
    assert t.dim() == 2 and t.stride(1) == 1 and t.shape[1] >= cols, (tuple(t.shape), t.stride(), cols)
    return max(t.stride(0), t.shape[1])


def _f32(t: torch.Tensor, *shape) -> torch.Tensor:
    assert t.dtype == torch.float32 and t.is_contiguous() and tuple(t.shape) == shape, (t.dtype, tuple(t.shape), shape)
    return t


# ------------------------------------------------------------------ residual stream
def _stream_args(x, y, w_post, w_last, tokens, embed, dtype):
    """Checks of what both forms of the residual step take; the sublayer's output as the C ABI wants it."""
    n, width = x.shape
    assert x.dtype == torch.float32
    y_stride = splits = split_stride = partial_stride = 0
    partial = None
    if isinstance(y, SplitKSum):
        y.check_alive()
        partial, y = y.partial, None
        assert partial.dtype == torch.float32 and partial.is_contiguous() and tuple(partial.shape[1:]) == (n, width)
        splits, split_stride, partial_stride = partial.shape[0], n * width, width
    elif y is not None:
        assert y.dtype == dtype and tuple(y.shape) == (n, width)
        y_stride = _rows(y, width)
    if y is not None or partial is not None:
        _f32(w_post, width)
    if w_last is not None:
        _f32(w_last, width)
    if tokens is not None:
        assert tokens.dtype == torch.int64 and tokens.is_contiguous() and tokens.numel() == n
        assert embed.dtype == dtype and embed.is_contiguous() and embed.shape[1] == width
    _require_gpu(x, *[t for t in (y, partial, w_post, w_last, tokens, embed) if t is not None])
    return _ptr(y), y_stride, _ptr(partial), splits, split_stride, partial_stride


def residual_norm(x: torch.Tensor, eps: float, *, y=None, w_post=None, w_pre=None, tokens=None, embed=None,
                  embed_scale: float = 1.0, dtype: torch.dtype = torch.bfloat16):
    """``x`` [rows, width] float32 is updated in place: the embedding of ``tokens`` is stored, or
    ``rms(y) * w_post`` added (``y`` may be an unreduced ``SplitKSum``).  Returns ``rms(x) * w_pre`` in ``dtype``,
    or None without ``w_pre``."""
    n, width = x.shape
    sub = _stream_args(x, y, w_post, w_pre, tokens, embed, dtype)
    out = torch.empty((n, width), dtype=dtype, device=x.device) if w_pre is not None else None
    rc = _lib.load().infer_residual_norm(
        ELEM[dtype], _ptr(tokens), _ptr(embed), float(embed_scale), embed.shape[0] if embed is not None else 0, *sub,
        _ptr(w_post), x.data_ptr(), _rows(x, width), _ptr(w_pre), _ptr(out), width, n, width, float(eps), _stream_ptr(x))
    _lib.check(rc, "residual_norm")
    return out


def post_norm(x: torch.Tensor, eps: float, *, y=None, w_post=None, alpha: float = 1.0, w_last=None, tokens=None, embed=None,
              embed_scale: float = 1.0, dtype: torch.dtype = torch.bfloat16) -> torch.Tensor:
    """``x`` [rows, width] float32 is updated in place: the embedding of ``tokens``, or
    ``rms(alpha * x + y) * w_post`` (``y`` may be an unreduced ``SplitKSum``).  Returns it in ``dtype``, with ``w_last``
    ``rms(x) * w_last`` instead."""
    n, width = x.shape
    sub = _stream_args(x, y, w_post, w_last, tokens, embed, dtype)
    out = torch.empty((n, width), dtype=dtype, device=x.device)
    rc = _lib.load().infer_post_norm(
        ELEM[dtype], _ptr(tokens), _ptr(embed), float(embed_scale), embed.shape[0] if embed is not None else 0, *sub,
        float(alpha), _ptr(w_post), x.data_ptr(), _rows(x, width), _ptr(w_last), out.data_ptr(), width, n, width, float(eps),
        _stream_ptr(x))
    _lib.check(rc, "post_norm")
    return out


@dataclass
class ExpertSum:
    """The output of a mixture of experts, not summed yet: for every token, ``weights`` times the rows ``places`` of ``rows`` (-1:
    the token's own row of ``h``), and ``shared`` (a tensor, a ``SplitKSum`` or None)."""
    rows: torch.Tensor
    places: torch.Tensor
    weights: torch.Tensor
    h: torch.Tensor
    shared: object = None


def pre_norm(x: torch.Tensor, w: torch.Tensor, eps: float, *, y=None, scale=None, first=None, step=None, tokens=None, embed=None,
             prev=None, bigram=None, multipliers=(0, 0), dtype: torch.dtype = torch.bfloat16) -> torch.Tensor:
    """``x`` [rows, width] float32 is updated in place: ``x + y * scale`` (``y`` a tensor, a ``SplitKSum`` or an ``ExpertSum``), plus
    ``first`` and ``step``; with ``tokens`` their embedding instead, plus the row of ``bigram`` that ``prev`` and the token
    address through ``multipliers``, which is written to ``first``, plus ``step``.  Returns ``rms(x) * w``."""
    n, width = x.shape
    _f32(w, width)
    experts = y if isinstance(y, ExpertSum) else None
    if experts is not None:
        y = experts.shared
        assert experts.rows.dtype == experts.h.dtype == dtype and experts.rows.is_contiguous() and experts.rows.shape[1] == width
        assert experts.places.dtype == torch.int32 and experts.places.is_contiguous() and experts.places.shape[0] == n
        _f32(experts.weights, *experts.places.shape)
        assert tuple(experts.h.shape) == (n, width)
    sub = _stream_args(x, y, scale if scale is not None else w, None, tokens, embed, dtype)
    for vector in (scale, step):
        if vector is not None:
            _f32(vector, width)
    if first is not None:
        _f32(first, n, width)
    buckets = 0
    if bigram is not None:
        assert bigram.dtype == dtype and bigram.is_contiguous() and bigram.shape[1] == width
        assert prev.dtype == torch.int64 and prev.is_contiguous() and prev.numel() == n
        buckets = bigram.shape[0] - 1
    _require_gpu(x, w, *[t for t in (scale, first, step, prev, bigram) if t is not None])
    out = torch.empty((n, width), dtype=dtype, device=x.device)
    e = experts
    rc = _lib.load().infer_pre_norm(
        ELEM[dtype], _ptr(tokens), _ptr(embed), embed.shape[0] if embed is not None else 0, _ptr(prev), _ptr(bigram), buckets,
        multipliers[0], multipliers[1], *sub, *((e.rows.data_ptr(), e.places.data_ptr(), e.weights.data_ptr(), e.places.shape[1],
                                                 e.rows.shape[0], e.h.data_ptr(), _rows(e.h, width)) if e is not None
                                                else (None, None, None, 0, 0, None, 0)),
        _ptr(scale), _ptr(first), _ptr(step), x.data_ptr(), _rows(x, width), w.data_ptr(), out.data_ptr(), width, n, width, float(eps),
        _stream_ptr(x))
    _lib.check(rc, "pre_norm")
    return out


def softcap(x: torch.Tensor, cap: float, scale: float = 1.0) -> torch.Tensor:
    """``cap * tanh(scale * x / cap)`` in float32."""
    n, cols = x.shape
    out = torch.empty((n, cols), dtype=torch.float32, device=x.device)
    _require_gpu(x)
    _lib.check(_lib.load().infer_softcap(ELEM[x.dtype], x.data_ptr(), _rows(x, cols), out.data_ptr(), n, cols, float(cap), float(scale),
                                         _stream_ptr(x)), "softcap")
    return out


@dataclass(frozen=True)
class TanhNorm:
    """``tanh(alpha * x) * weight + bias``: a norm without statistics."""
    alpha: float
    weight: torch.Tensor
    bias: torch.Tensor


def tanh_norm(x: torch.Tensor, norm: TanhNorm, *, y=None, bias=None, tokens=None, embed=None, embed_scale: float = 1.0,
              embed_norm: TanhNorm | None = None, dtype: torch.dtype = torch.bfloat16) -> torch.Tensor:
    """``x`` [rows, width] float32 is updated in place: ``x + y + bias`` (``y`` a tensor or a ``SplitKSum``), or with ``tokens`` the
    ``embed_norm`` of their scaled embedding.  Returns its ``norm``."""
    n, width = x.shape
    sub = _stream_args(x, y, norm.weight, norm.weight, tokens, embed, dtype)
    vectors = [norm.weight, norm.bias] + ([embed_norm.weight, embed_norm.bias] if tokens is not None else []) + ([bias] if bias is not None else [])
    for v in vectors:
        _f32(v, width)
    _require_gpu(x, *vectors)
    out = torch.empty((n, width), dtype=dtype, device=x.device)
    first = embed_norm if tokens is not None else TanhNorm(1.0, None, None)
    rc = _lib.load().infer_tanh_norm(
        ELEM[dtype], _ptr(tokens), _ptr(embed), embed.shape[0] if embed is not None else 0, float(embed_scale), float(first.alpha),
        _ptr(first.weight), _ptr(first.bias), *sub, _ptr(bias), x.data_ptr(), _rows(x, width), float(norm.alpha), norm.weight.data_ptr(),
        norm.bias.data_ptr(), out.data_ptr(), width, n, width, _stream_ptr(x))
    _lib.check(rc, "tanh_norm")
    return out


def xielu(x: torch.Tensor, bias: torch.Tensor, p: float, q: float) -> torch.Tensor:
    """Of ``z = x + bias``: ``p z^2 + z / 2`` where it is positive, ``q (e^z - 1 - z) + z / 2`` elsewhere."""
    n, cols = x.shape
    _f32(bias, cols)
    out = torch.empty((n, cols), dtype=x.dtype, device=x.device)
    _require_gpu(x, bias)
    _lib.check(_lib.load().infer_xielu(ELEM[x.dtype], x.data_ptr(), _rows(x, cols), bias.data_ptr(), float(p), float(q), out.data_ptr(),
                                       cols, n, cols, _stream_ptr(x)), "xielu")
    return out


def _gated(entry: str, x: torch.Tensor, *constants: float) -> torch.Tensor:
    d = x.shape[1] // 2
    out = torch.empty((x.shape[0], d), dtype=x.dtype, device=x.device)
    _require_gpu(x)
    rc = getattr(_lib.load(), entry)(ELEM[x.dtype], out.data_ptr(), d, x.data_ptr(), _rows(x, 2 * d), x.shape[0], d, *constants,
                                       _stream_ptr(x))
    _lib.check(rc, entry)
    return out


def gelu_tanh_and_mul(x: torch.Tensor) -> torch.Tensor:
    """``gelu_tanh(x[:, :d]) * x[:, d:]``."""
    return _gated("infer_gelu_tanh_and_mul", x)


def silu_and_mul(x: torch.Tensor) -> torch.Tensor:
    """``silu(x[:, :d]) * x[:, d:]``."""
    return _gated("infer_silu_and_mul", x)


def clamped_gate_and_mul(x: torch.Tensor, limit: float) -> torch.Tensor:
    """``g * sigmoid(1.702 g) * (u + 1)`` with ``g = min(x[:, :d], limit)`` and ``u = clamp(x[:, d:], -limit, limit)``."""
    return _gated("infer_clamped_gate_and_mul", x, float(limit))


# ------------------------------------------------------------------ latent attention
def latent_front(proj, heads, dim, rot, rot_dims, kv_off, rank, c_norm, eps, table, positions, slots, cache, rank_pad,
                 qx, qx_rows) -> None:
    """Norm of the latent, rotary positions and the append of one cache row per token; ``cache`` is
    [blocks, block_size, row], ``qx`` [>= qx_rows, heads, row]."""
    n = proj.shape[0]
    row = cache.shape[2]
    _f32(c_norm, rank)
    assert table.dtype == torch.float32 and table.is_contiguous() and table.shape[1:] == (rot_dims // 2, 2)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == n
    assert slots.dtype == torch.int32 and slots.is_contiguous() and slots.numel() == n
    assert cache.dtype == proj.dtype and cache.is_contiguous()
    assert qx_rows == 0 or (qx.dtype == proj.dtype and qx.is_contiguous() and tuple(qx.shape[1:]) == (heads, row)
                            and qx.shape[0] >= qx_rows)
    _require_gpu(proj, c_norm, table, positions, slots, cache)
    rc = _lib.load().infer_latent_front(
        ELEM[proj.dtype], proj.data_ptr(), _rows(proj, kv_off + rank + rot), heads, dim, rot, rot_dims, kv_off, rank,
        c_norm.data_ptr(), float(eps), table.data_ptr(), table.shape[0], positions.data_ptr(), slots.data_ptr(),
        cache.data_ptr(), rank_pad, row, cache.shape[0] * cache.shape[1], _ptr(qx) if qx_rows else None, qx_rows, n,
        _stream_ptr(proj))
    _lib.check(rc, "latent_front")


def head_matmul(x, w, out, n: int, k: int, gate=None) -> None:
    """``out[m, h, :n] = w[h, :n, :k] x[m, h, :k]`` (times ``sigmoid(gate[m, h])``) on 3-D views with a contiguous last
    axis; ``w`` [heads, n padded to 16, k padded to 32] is padded with zeros."""
    m, heads = x.shape[:2]
    assert x.dtype == w.dtype == out.dtype and out.shape[:2] == (m, heads) and w.shape[0] == heads
    assert x.stride(2) == 1 and out.stride(2) == 1 and w.is_contiguous()
    assert x.shape[2] >= k and out.shape[2] >= n and w.shape[1] >= (n + 15) // 16 * 16 and w.shape[2] >= k
    if gate is not None:
        assert gate.dtype == x.dtype and gate.shape[0] == m and gate.shape[1] >= heads and gate.stride(1) == 1
    _require_gpu(x, w, out)
    rc = _lib.load().infer_head_matmul(
        ELEM[x.dtype], x.data_ptr(), x.stride(0), x.stride(1), w.data_ptr(), w.stride(0), w.shape[2], out.data_ptr(),
        out.stride(0), out.stride(1), _ptr(gate), max(gate.stride(0), heads) if gate is not None else 0, m, heads, n, k,
        _stream_ptr(x))
    _lib.check(rc, "head_matmul")


def latent_attention(qx, cache, block_table, ctx, scale: float, rank_pad: int, row_seq=None, max_keys=None,
                     splits: int = 0) -> torch.Tensor:
    """``qx`` [rows, heads, row] against the first ``ctx[r]`` cached rows of the sequence in block-table row
    ``row_seq[r]`` (default ``r``).  Returns the weighted latents [rows, heads, rank_pad].  ``max_keys`` bounds ``ctx`` for the
    choice of ``splits`` (default: what a block-table row can address)."""
    rows, heads, row = qx.shape
    nblk, bs, crow = cache.shape
    assert qx.is_contiguous() and cache.is_contiguous() and cache.dtype == qx.dtype and crow == row
    assert block_table.dtype == torch.int32 and block_table.dim() == 2 and block_table.stride(1) == 1
    assert ctx.dtype == torch.int32 and ctx.is_contiguous() and ctx.numel() == rows
    if row_seq is None:
        assert block_table.shape[0] >= rows
    else:
        assert row_seq.dtype == torch.int32 and row_seq.is_contiguous() and row_seq.numel() == rows
    _require_gpu(qx, cache, block_table, ctx)
    lib = _lib.load()
    elem, cols = ELEM[qx.dtype], block_table.shape[1]
    if splits <= 0:
        splits = lib.infer_latent_attention_splits(elem, rows, heads, row, rank_pad, bs, max_keys or cols * bs)
    out = torch.empty((rows, heads, rank_pad), dtype=qx.dtype, device=qx.device)
    need = rows * splits * heads * (rank_pad + 2) if splits > 1 else 0
    ws = torch.empty(need, dtype=torch.float32, device=qx.device) if need else None
    rc = lib.infer_latent_attention(elem, qx.data_ptr(), cache.data_ptr(), row, rank_pad, block_table.data_ptr(),
                                    max(block_table.stride(0), cols), cols, bs, nblk, _ptr(row_seq), ctx.data_ptr(), rows,
                                    heads, float(scale), splits, out.data_ptr(), _ptr(ws), need, _stream_ptr(qx))
    _lib.check(rc, "latent_attention")
    return out


def latent_gather(cache, block_table, seqs, cu_k, total: int, max_keys: int) -> torch.Tensor:
    """The cached rows of the sequences in block-table rows ``seqs`` as dense rows [total, row]."""
    nblk, bs, row = cache.shape
    assert cache.dtype == torch.bfloat16 and cache.is_contiguous()
    assert block_table.dtype == torch.int32 and block_table.stride(1) == 1
    for t in (seqs, cu_k):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert cu_k.numel() == seqs.numel() + 1
    _require_gpu(cache, block_table, seqs, cu_k)
    out = torch.empty((total, row), dtype=cache.dtype, device=cache.device)
    rc = _lib.load().infer_latent_gather(cache.data_ptr(), row, bs, nblk, block_table.data_ptr(),
                                         max(block_table.stride(0), block_table.shape[1]), block_table.shape[1],
                                         seqs.data_ptr(), cu_k.data_ptr(), seqs.numel(), max_keys, out.data_ptr(),
                                         _stream_ptr(cache))
    _lib.check(rc, "latent_gather")
    return out


def latent_prefill_supported(dim: int, rot: int, vdim: int) -> bool:
    """Whether the dense-key prefill kernel serves these sizes."""
    return bool(_lib.load().infer_latent_prefill_supported(dim, rot, vdim))


def latent_prefill(q, kp, kr, v, gate, out, cu_q, cu_k, max_seqlen_q: int, heads, dim, rot, vdim, scale) -> None:
    """Causal attention of whole portions over dense keys and values (all bf16, 2-D views)."""
    for t in (q, kp, kr, v, gate, out):
        assert t.dtype == torch.bfloat16
    for t in (cu_q, cu_k):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert cu_q.numel() == cu_k.numel() and kp.shape[0] == kr.shape[0] == v.shape[0]
    assert q.shape[0] == gate.shape[0] == out.shape[0]
    _require_gpu(q, kp, kr, v, gate, out, cu_q, cu_k)
    rc = _lib.load().infer_latent_prefill(
        q.data_ptr(), _rows(q, heads * (dim + rot)), kp.data_ptr(), kp.stride(0), kr.data_ptr(), kr.stride(0), v.data_ptr(),
        v.stride(0), gate.data_ptr(), max(gate.stride(0), heads), out.data_ptr(), _rows(out, heads * vdim), cu_q.data_ptr(),
        cu_k.data_ptr(), cu_q.numel() - 1, int(max_seqlen_q), heads, dim, rot, vdim, float(scale), _stream_ptr(q))
    _lib.check(rc, "latent_prefill")


# ------------------------------------------------------------------ grouped attention
def grouped_front(proj, heads, kv_heads, dim, vdim, k_off, v_off, bias, q_norm, k_norm, eps, table, rot_dims, positions, slots,
                  cache, dim_pad, vdim_pad, qx, qx_rows) -> None:
    """Biases, norms over the whole projections, rotary positions and the append of keys and values; ``cache`` is
    [blocks, kv_heads, block_size, vdim_pad + dim_pad], ``qx`` [>= qx_rows, heads, dim_pad].  ``kv_heads`` 0: q alone."""
    n = proj.shape[0]
    cols = v_off + kv_heads * vdim if kv_heads else heads * dim
    if bias is not None:
        assert bias.dtype == torch.float32 and bias.is_contiguous() and bias.numel() >= cols
    if q_norm is not None:
        _f32(q_norm, heads * dim)
    if kv_heads and k_norm is not None:
        _f32(k_norm, kv_heads * dim)
    assert table.dtype == torch.float32 and table.is_contiguous() and table.shape[1:] == (rot_dims // 2, 2)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == n
    assert slots.dtype == torch.int32 and slots.is_contiguous() and slots.numel() == n
    assert cache.dtype == proj.dtype and cache.is_contiguous() and cache.shape[3] == dim_pad + vdim_pad
    assert kv_heads in (0, cache.shape[1])
    assert qx_rows == 0 or (qx.dtype == proj.dtype and qx.is_contiguous() and tuple(qx.shape[1:]) == (heads, dim_pad)
                            and qx.shape[0] >= qx_rows)
    _require_gpu(proj, table, positions, slots, cache)
    rc = _lib.load().infer_grouped_front(
        ELEM[proj.dtype], proj.data_ptr(), _rows(proj, cols), heads, kv_heads, dim, vdim, k_off, v_off, _ptr(bias), _ptr(q_norm),
        _ptr(k_norm) if kv_heads else None, float(eps), table.data_ptr() if rot_dims else None, rot_dims, table.shape[0],
        positions.data_ptr(), slots.data_ptr(), cache.data_ptr(), cache.shape[2], dim_pad, vdim_pad,
        cache.shape[0] * cache.shape[2], _ptr(qx) if qx_rows else None, qx_rows, n, _stream_ptr(proj))
    _lib.check(rc, "grouped_front")


def grouped_attention(qx, cache, block_table, ctx, scale: float, vdim: int, out, sink=None, gate=None, row_seq=None, max_keys=None,
                      splits: int = 0) -> None:
    """``qx`` [rows, heads, dim_pad] against the first ``ctx[r]`` keys of the sequence in block-table row ``row_seq[r]``
    (default ``r``); ``out`` [rows, heads * vdim].  ``sink`` [heads] float32, ``gate`` [rows, heads]."""
    rows, heads, dim_pad = qx.shape
    nblk, kv_heads, bs, crow = cache.shape
    vdim_pad = crow - dim_pad
    assert qx.is_contiguous() and cache.is_contiguous() and cache.dtype == qx.dtype == out.dtype and 0 < vdim <= vdim_pad
    assert block_table.dtype == torch.int32 and block_table.dim() == 2 and block_table.stride(1) == 1
    assert ctx.dtype == torch.int32 and ctx.is_contiguous() and ctx.numel() == rows and out.shape[0] == rows
    if row_seq is None:
        assert block_table.shape[0] >= rows
    else:
        assert row_seq.dtype == torch.int32 and row_seq.is_contiguous() and row_seq.numel() == rows
    if sink is not None:
        _f32(sink, heads)
    if gate is not None:
        assert gate.dtype == qx.dtype and gate.shape[0] == rows and gate.shape[1] >= heads and gate.stride(1) == 1
    _require_gpu(qx, cache, block_table, ctx, out)
    lib = _lib.load()
    elem, cols = ELEM[qx.dtype], block_table.shape[1]
    if splits <= 0:
        splits = lib.infer_grouped_attention_splits(elem, rows, heads, kv_heads, dim_pad, vdim_pad, bs, max_keys or cols * bs)
    need = rows * splits * heads * (vdim_pad + 2) if splits > 1 else 0
    ws = torch.empty(need, dtype=torch.float32, device=qx.device) if need else None
    rc = lib.infer_grouped_attention(
        elem, qx.data_ptr(), cache.data_ptr(), dim_pad, vdim_pad, block_table.data_ptr(), max(block_table.stride(0), cols), cols, bs,
        nblk, _ptr(row_seq), ctx.data_ptr(), rows, heads, kv_heads, float(scale), _ptr(sink), _ptr(gate),
        max(gate.stride(0), heads) if gate is not None else 0, splits, out.data_ptr(), _rows(out, heads * vdim), vdim, _ptr(ws), need,
        _stream_ptr(qx))
    _lib.check(rc, "grouped_attention")


def grouped_gather(cache, block_table, seqs, cu_k, total: int, max_keys: int) -> torch.Tensor:
    """The cached rows of the sequences in block-table rows ``seqs`` as dense rows [total, kv_heads, row]."""
    nblk, kv_heads, bs, row = cache.shape
    assert cache.dtype == torch.bfloat16 and cache.is_contiguous()
    assert block_table.dtype == torch.int32 and block_table.stride(1) == 1
    for t in (seqs, cu_k):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert cu_k.numel() == seqs.numel() + 1
    _require_gpu(cache, block_table, seqs, cu_k)
    out = torch.empty((total, kv_heads, row), dtype=cache.dtype, device=cache.device)
    rc = _lib.load().infer_grouped_gather(cache.data_ptr(), row, kv_heads, bs, nblk, block_table.data_ptr(),
                                          max(block_table.stride(0), block_table.shape[1]), block_table.shape[1],
                                          seqs.data_ptr(), cu_k.data_ptr(), seqs.numel(), max_keys, out.data_ptr(),
                                          _stream_ptr(cache))
    _lib.check(rc, "grouped_gather")
    return out


def grouped_prefill_supported(dim: int, vdim: int) -> bool:
    """Whether the dense-key prefill kernel serves these sizes."""
    return bool(_lib.load().infer_grouped_prefill_supported(dim, vdim))


def grouped_prefill(q, k, v, sink, gate, out, cu_q, cu_k, max_seqlen_q: int, heads, dim, vdim, scale) -> None:
    """Causal attention of whole portions: ``q`` [tokens, heads * dim], ``k``/``v`` [keys, kv_heads, dim / vdim] (views of dense
    rows), ``gate`` [tokens, heads], ``out`` [tokens, heads * vdim], all bf16; ``sink`` [heads] float32 or None."""
    for t in (q, k, v, gate, out):
        assert t.dtype == torch.bfloat16
    for t in (cu_q, cu_k):
        assert t.dtype == torch.int32 and t.is_contiguous()
    kv_heads = k.shape[1]
    assert k.dim() == v.dim() == 3 and k.stride(2) == v.stride(2) == 1 and k.shape[:2] == v.shape[:2]
    assert k.shape[2] >= dim and v.shape[2] >= vdim and cu_q.numel() == cu_k.numel()
    assert q.shape[0] == gate.shape[0] == out.shape[0]
    if sink is not None:
        _f32(sink, heads)
    _require_gpu(q, k, v, gate, out, cu_q, cu_k)
    rc = _lib.load().infer_grouped_prefill(
        q.data_ptr(), _rows(q, heads * dim), k.data_ptr(), k.stride(0), k.stride(1), v.data_ptr(), v.stride(0), v.stride(1), _ptr(sink),
        gate.data_ptr(), max(gate.stride(0), heads), out.data_ptr(), _rows(out, heads * vdim), cu_q.data_ptr(), cu_k.data_ptr(),
        cu_q.numel() - 1, int(max_seqlen_q), heads, kv_heads, dim, vdim, float(scale), _stream_ptr(q))
    _lib.check(rc, "grouped_prefill")


# ------------------------------------------------------------------ masked attention
MASKS = {None: 0, "chunk": 1, "window": 2}


@dataclass(frozen=True)
class MaskedShape:
    """Sizes and constants of masked attention.  ``maps`` 2: the difference of two attentions over the same values
    (``lam``, and ``out_scale`` behind its norm); otherwise ``out_scale`` multiplies the output."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    maps: int = 1
    mask: str | None = None
    mask_size: int = 1
    distance_bias: bool = False
    out_scale: float = 1.0
    lam: float = 0.0
    eps: float = 0.0
    rot_dims: int = 0

    @property
    def key_pad(self) -> int:
        return -(-self.maps * self.dim // 32) * 32

    @property
    def vdim_pad(self) -> int:
        return -(-self.vdim // 32) * 32


def head_front(s: MaskedShape, proj, offsets, bias, q_norm, k_norm, table, positions, slots, cache, qx, qx_rows: int) -> None:
    """Biases, norms per head, rotary positions and the append of keys and values; ``cache`` is
    [blocks, kv_heads, block_size, vdim_pad + key_pad], ``qx`` [>= qx_rows, heads * maps, key_pad]."""
    n = proj.shape[0]
    cols = max(offsets[0] + s.heads * s.maps * s.dim, offsets[1] + s.kv_heads * s.maps * s.dim, offsets[2] + s.kv_heads * s.vdim)
    if bias is not None:
        assert bias.dtype == torch.float32 and bias.is_contiguous() and bias.numel() >= cols
    for norm in (q_norm, k_norm):
        if norm is not None:
            _f32(norm, s.dim)
    if s.rot_dims:
        assert table.dtype == torch.float32 and table.is_contiguous() and table.shape[1:] == (s.rot_dims // 2, 2)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == n
    assert slots.dtype == torch.int32 and slots.is_contiguous() and slots.numel() == n
    assert cache.dtype == proj.dtype and cache.is_contiguous() and cache.shape[1] == s.kv_heads and cache.shape[3] == s.key_pad + s.vdim_pad
    assert qx_rows == 0 or (qx.dtype == proj.dtype and qx.is_contiguous() and tuple(qx.shape[1:]) == (s.heads * s.maps, s.key_pad)
                            and qx.shape[0] >= qx_rows)
    _require_gpu(proj, positions, slots, cache)
    rc = _lib.load().infer_head_front(
        ELEM[proj.dtype], proj.data_ptr(), _rows(proj, cols), s.heads, s.kv_heads, s.maps, s.dim, s.vdim, *offsets, _ptr(bias),
        _ptr(q_norm), _ptr(k_norm), float(s.eps), _ptr(table) if s.rot_dims else None, s.rot_dims, table.shape[0] if s.rot_dims else 1,
        positions.data_ptr(), slots.data_ptr(), cache.data_ptr(), cache.shape[2], s.key_pad, s.vdim_pad,
        cache.shape[0] * cache.shape[2], _ptr(qx) if qx_rows else None, qx_rows, n, _stream_ptr(proj))
    _lib.check(rc, "head_front")


def _optional_heads(sink, gate, s: MaskedShape, rows: int, dtype) -> tuple:
    if sink is not None:
        _f32(sink, s.heads)
    if gate is not None:
        assert gate.dtype == dtype and gate.shape[0] == rows and gate.shape[1] >= s.heads and gate.stride(1) == 1
    return _ptr(sink), _ptr(gate), max(gate.stride(0), s.heads) if gate is not None else 0


def masked_attention(s: MaskedShape, qx, cache, block_table, ctx, out, sink=None, gate=None, row_seq=None, max_keys=None,
                     splits: int = 0) -> None:
    """``qx`` [rows, heads * maps, key_pad] against what the mask shows of the first ``ctx[r]`` keys of the sequence in block-table
    row ``row_seq[r]`` (default ``r``); ``out`` [rows, heads * vdim].  ``sink`` [heads] float32, ``gate`` [rows, heads]."""
    rows, heads = qx.shape[:2]
    nblk, kv_heads, bs, crow = cache.shape
    assert qx.is_contiguous() and cache.is_contiguous() and cache.dtype == qx.dtype == out.dtype
    assert heads == s.heads * s.maps and qx.shape[2] == s.key_pad and kv_heads == s.kv_heads and crow == s.key_pad + s.vdim_pad
    assert block_table.dtype == torch.int32 and block_table.dim() == 2 and block_table.stride(1) == 1
    assert ctx.dtype == torch.int32 and ctx.is_contiguous() and ctx.numel() == rows and out.shape[0] == rows
    if row_seq is None:
        assert block_table.shape[0] >= rows
    else:
        assert row_seq.dtype == torch.int32 and row_seq.is_contiguous() and row_seq.numel() == rows
    extra = _optional_heads(sink, gate, s, rows, qx.dtype)
    _require_gpu(qx, cache, block_table, ctx, out)
    lib = _lib.load()
    elem, cols = ELEM[qx.dtype], block_table.shape[1]
    if splits <= 0:
        keys = max_keys or cols * bs
        if s.mask is not None:
            keys = min(keys, s.mask_size + 31)           # whole tiles of keys are read
        splits = lib.infer_grouped_attention_splits(elem, rows, heads, kv_heads, s.key_pad, s.vdim_pad, bs, keys)
    need = rows * splits * heads * (s.vdim_pad + 2) if splits > 1 or s.maps == 2 else 0
    ws = torch.empty(need, dtype=torch.float32, device=qx.device) if need else None
    rc = lib.infer_masked_attention(
        elem, qx.data_ptr(), cache.data_ptr(), s.key_pad, s.vdim_pad, block_table.data_ptr(), max(block_table.stride(0), cols), cols, bs,
        nblk, _ptr(row_seq), ctx.data_ptr(), rows, s.heads, s.kv_heads, s.maps, float(s.scale), MASKS[s.mask], s.mask_size,
        int(s.distance_bias), *extra, float(s.out_scale), float(s.lam), float(s.eps), splits, out.data_ptr(),
        _rows(out, s.heads * s.vdim), s.vdim, _ptr(ws), need, _stream_ptr(qx))
    _lib.check(rc, "masked_attention")


def masked_gather(s: MaskedShape, cache, block_table, seqs, cu_q, cu_k, total: int, max_keys: int) -> torch.Tensor:
    """The cached rows of the sequences in block-table rows ``seqs`` as dense rows [total, kv_heads, row]; rows in front of what the
    first query of a portion sees are left out."""
    nblk, kv_heads, bs, row = cache.shape
    assert cache.dtype == torch.bfloat16 and cache.is_contiguous()
    assert block_table.dtype == torch.int32 and block_table.stride(1) == 1
    for t in (seqs, cu_q, cu_k):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert cu_q.numel() == cu_k.numel() == seqs.numel() + 1
    _require_gpu(cache, block_table, seqs, cu_q, cu_k)
    out = torch.empty((total, kv_heads, row), dtype=cache.dtype, device=cache.device)
    rc = _lib.load().infer_masked_gather(cache.data_ptr(), row, kv_heads, bs, nblk, block_table.data_ptr(),
                                         max(block_table.stride(0), block_table.shape[1]), block_table.shape[1], seqs.data_ptr(),
                                         cu_q.data_ptr(), cu_k.data_ptr(), seqs.numel(), max_keys, MASKS[s.mask], s.mask_size,
                                         out.data_ptr(), _stream_ptr(cache))
    _lib.check(rc, "masked_gather")
    return out


def masked_prefill_supported(s: MaskedShape) -> bool:
    """Whether the dense-key prefill kernel serves these sizes."""
    return bool(_lib.load().infer_masked_prefill_supported(s.maps, s.dim, s.vdim))


def masked_prefill(s: MaskedShape, q, rows, out, cu_q, cu_k, max_seqlen_q: int, sink=None, gate=None) -> None:
    """Whole portions: ``q`` [tokens, heads * maps * dim], ``rows`` [keys, kv_heads, row] dense rows, ``gate`` [tokens, heads], ``out``
    [tokens, heads * vdim], all bf16; ``sink`` [heads] float32."""
    for t in (q, rows, out):
        assert t.dtype == torch.bfloat16
    for t in (cu_q, cu_k):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert rows.is_contiguous() and rows.shape[1:] == (s.kv_heads, s.key_pad + s.vdim_pad) and cu_q.numel() == cu_k.numel()
    assert q.shape[0] == out.shape[0]
    k = rows[:, :, s.vdim_pad:]
    extra = _optional_heads(sink, gate, s, q.shape[0], q.dtype)
    _require_gpu(q, rows, out, cu_q, cu_k)
    rc = _lib.load().infer_masked_prefill(
        q.data_ptr(), _rows(q, s.heads * s.maps * s.dim), k.data_ptr(), k.stride(0), k.stride(1), rows.data_ptr(), rows.stride(0),
        rows.stride(1), *extra, out.data_ptr(), _rows(out, s.heads * s.vdim), cu_q.data_ptr(), cu_k.data_ptr(), cu_q.numel() - 1,
        int(max_seqlen_q), s.heads, s.kv_heads, s.maps, s.dim, s.vdim, float(s.scale), MASKS[s.mask], s.mask_size, int(s.distance_bias),
        float(s.out_scale), float(s.lam), float(s.eps), _stream_ptr(q))
    _lib.check(rc, "masked_prefill")


# ------------------------------------------------------------------ talking-heads attention
@dataclass(frozen=True)
class TalkShape:
    """Sizes and constants of attention whose heads mix their weights.  ``temp_every`` 0: no temperature of the queries."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    eps: float
    norm_values: bool = True
    temp_coef: float = 0.0
    temp_every: float = 0.0
    out_scale: float = 1.0

    @property
    def key_pad(self) -> int:
        return -(-self.dim // 32) * 32

    @property
    def vdim_pad(self) -> int:
        return -(-self.vdim // 32) * 32

    def max_score(self, positions: int) -> float:
        """A bound of the scores at the first ``positions`` positions, with some room for rounding: queries and keys have the root mean
        square one (or less)."""
        temp = 1.0
        if self.temp_every > 0:
            temp = max(1.0, abs(1.0 + self.temp_coef * math.log(positions // self.temp_every + 1.0)))
        return 1.05 * abs(self.scale) * self.dim * temp


def _talk_pages(s: TalkShape, keys, values, dtype):
    """(blocks, block size) of checked pages (``cache.TilePages``)."""
    assert keys.dtype == values.dtype == dtype and keys.is_contiguous() and values.is_contiguous() and keys.shape[:3] == values.shape[:3]
    assert keys.shape[1] == s.kv_heads and tuple(keys.shape[3:]) == (s.key_pad // 8, 32, 8)
    assert tuple(values.shape[3:]) == (s.vdim_pad // 16, 4, 16, 8)
    return keys.shape[0], 32 * keys.shape[2]


def unit_head_front(s: TalkShape, proj, offsets, positions, slots, keys, values, qx, qx_rows: int) -> None:
    """Norms per head, the temperature of the queries and the append of keys and values to pages of tiles; ``qx``
    [>= qx_rows, heads, key_pad]."""
    n = proj.shape[0]
    blocks, bs = _talk_pages(s, keys, values, proj.dtype)
    cols = max(offsets[0] + s.heads * s.dim, offsets[1] + s.kv_heads * s.dim, offsets[2] + s.kv_heads * s.vdim)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == n
    assert slots.dtype == torch.int32 and slots.is_contiguous() and slots.numel() == n
    assert qx_rows == 0 or (qx.dtype == proj.dtype and qx.is_contiguous() and tuple(qx.shape[1:]) == (s.heads, s.key_pad)
                            and qx.shape[0] >= qx_rows)
    _require_gpu(proj, positions, slots, keys, values)
    rc = _lib.load().infer_unit_head_front(
        ELEM[proj.dtype], proj.data_ptr(), _rows(proj, cols), s.heads, s.kv_heads, s.dim, s.vdim, *offsets, float(s.eps), int(s.norm_values),
        float(s.temp_coef), float(s.temp_every), positions.data_ptr(), slots.data_ptr(), keys.data_ptr(), values.data_ptr(), bs, s.key_pad,
        s.vdim_pad, blocks * bs, _ptr(qx) if qx_rows else None, qx_rows, n, _stream_ptr(proj))
    _lib.check(rc, "unit_head_front")


TALK_SCORES = 1 << 28          # scores that one call may keep at a time (1 GiB of float32)


def talking_attention(s: TalkShape, qx, keys, values, talk, block_table, ctx, out, row_seq=None, max_keys=None, splits: int = 0) -> None:
    """``qx`` [rows, heads, key_pad] against the first ``ctx[r]`` keys of the sequence in block-table row ``row_seq[r]`` (default
    ``r``); ``talk`` [heads, heads]; ``out`` [rows, heads * vdim].  ``max_keys`` bounds ``ctx`` (default: what a block-table row can
    address).  Many rows with many keys run in turns, so that their scores fit a workspace."""
    rows = qx.shape[0]
    blocks, bs = _talk_pages(s, keys, values, qx.dtype)
    assert qx.is_contiguous() and tuple(qx.shape[1:]) == (s.heads, s.key_pad) and out.dtype == qx.dtype and out.shape[0] == rows
    assert talk.dtype == qx.dtype and talk.is_contiguous() and tuple(talk.shape) == (s.heads, s.heads)
    assert block_table.dtype == torch.int32 and block_table.dim() == 2 and block_table.stride(1) == 1
    assert ctx.dtype == torch.int32 and ctx.is_contiguous() and ctx.numel() == rows
    if row_seq is None:
        assert block_table.shape[0] >= rows
    else:
        assert row_seq.dtype == torch.int32 and row_seq.is_contiguous() and row_seq.numel() == rows
    _require_gpu(qx, keys, values, talk, block_table, ctx, out)
    lib, elem, cols = _lib.load(), ELEM[qx.dtype], block_table.shape[1]
    max_keys = min(max_keys or cols * bs, cols * bs)
    turn = max(1, min(rows, TALK_SCORES // (s.heads * max_keys)))
    forced = splits
    for lo in range(0, rows, turn):
        n = min(turn, rows - lo)
        splits = forced or lib.infer_talking_attention_splits(elem, n, s.heads, s.kv_heads, s.key_pad, s.vdim_pad, bs, max_keys)
        need = lib.infer_talking_attention_workspace_floats(n, s.heads, s.vdim_pad, splits, max_keys)
        ws = torch.empty(need, dtype=torch.float32, device=qx.device)
        table = block_table[lo:] if row_seq is None else block_table
        rc = lib.infer_talking_attention(
            elem, qx[lo:].data_ptr(), keys.data_ptr(), values.data_ptr(), s.key_pad, s.vdim_pad, table.data_ptr(), max(block_table.stride(0), cols),
            cols, bs, blocks, None if row_seq is None else row_seq[lo:].data_ptr(), ctx[lo:].data_ptr(), n, s.heads, s.kv_heads, float(s.scale),
            talk.data_ptr(), float(s.out_scale), splits, max_keys, out[lo:].data_ptr(), _rows(out, s.heads * s.vdim), s.vdim, ws.data_ptr(), need,
            _stream_ptr(qx))
        _lib.check(rc, "talking_attention")


def talking_prefill_supported(s: TalkShape) -> bool:
    """Whether the kernels for whole portions serve these sizes."""
    return bool(_lib.load().infer_talking_prefill_supported(s.heads, s.dim, s.vdim))


def talking_prefill(s: TalkShape, q, keys, values, talk, block_table, seqs, cu_q, cu_k, max_seqlen_q: int, max_keys: int, out,
                    max_score=None) -> None:
    """Whole portions: ``q`` [tokens, heads * dim] (behind ``unit_head_front``) are the last tokens of the sequences in block-table rows
    ``seqs``, whose numbers of keys (at most ``max_keys``) ``cu_k`` sums up; ``out`` [tokens, heads * vdim], all bf16.  ``max_score``: no score is larger
    (None: nobody knows); a small bound spares the search for maxima."""
    blocks, bs = _talk_pages(s, keys, values, torch.bfloat16)
    assert q.dtype == out.dtype == talk.dtype == torch.bfloat16 and q.shape[0] == out.shape[0]
    assert talk.is_contiguous() and tuple(talk.shape) == (s.heads, s.heads)
    assert block_table.dtype == torch.int32 and block_table.dim() == 2 and block_table.stride(1) == 1
    for t in (seqs, cu_q, cu_k):
        assert t.dtype == torch.int32 and t.is_contiguous()
    assert cu_q.numel() == cu_k.numel() == seqs.numel() + 1
    _require_gpu(q, keys, values, talk, block_table, seqs, cu_q, cu_k, out)
    tokens, cols = q.shape[0], block_table.shape[1]
    lib = _lib.load()
    ws = torch.empty(lib.infer_talking_prefill_workspace_floats(s.heads, s.vdim, seqs.numel(), tokens, int(max_seqlen_q), int(max_keys)),
                     dtype=torch.float32, device=q.device)
    rc = lib.infer_talking_prefill(
        q.data_ptr(), _rows(q, s.heads * s.dim), keys.data_ptr(), values.data_ptr(), s.key_pad, s.vdim_pad, block_table.data_ptr(),
        max(block_table.stride(0), cols), cols, bs, blocks, seqs.data_ptr(), cu_q.data_ptr(), cu_k.data_ptr(), seqs.numel(), tokens,
        int(max_seqlen_q), int(max_keys), s.heads, s.kv_heads, s.dim, s.vdim, float(s.scale), talk.data_ptr(), float(s.out_scale),
        float("inf") if max_score is None else float(max_score), out.data_ptr(), _rows(out, s.heads * s.vdim), ws.data_ptr(), ws.numel(),
        _stream_ptr(q))
    _lib.check(rc, "talking_prefill")


# ------------------------------------------------------------------ selective state space
@dataclass(frozen=True)
class StateSpaceShape:
    """Sizes and constants of a state-space layer; ``groups`` of heads share B and C, the norm has ``norm_parts`` parts."""
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int
    norm_parts: int
    eps: float

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state


def state_space(s: StateSpaceShape, proj, offsets, conv, conv_bias, dt_bias, a_log, d, norm, ring, state, slots, positions,
                decode_rows: int, spans, max_span: int, ring_slot, out) -> None:
    """``proj`` holds z, [x | B | C] and dt at the columns ``offsets``.  Rows below ``decode_rows`` advance the state of
    ``slots[r]`` by one token (negative: padding), the others belong to ``spans`` [.., 4] (first row, tokens, slot, first
    position); ``ring_slot`` [rows, 2] is a row's slot and the rows of its span that follow."""
    n = proj.shape[0]
    z, x, dt = offsets
    assert proj.dtype == out.dtype == ring.dtype and out.shape[0] == n
    _f32(conv, s.channels, s.taps)
    _f32(conv_bias, s.channels)
    for vector in (dt_bias, a_log, d):
        _f32(vector, s.heads)
    _f32(norm, s.inner)
    _f32(state, state.shape[0], s.heads, s.state, s.vdim)
    assert ring.is_contiguous() and tuple(ring.shape) == (state.shape[0], s.taps, s.channels)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == n
    if decode_rows:
        assert slots.dtype == torch.int32 and slots.is_contiguous() and slots.numel() >= decode_rows
    lib, elem = _lib.load(), ELEM[proj.dtype]
    num_spans, need, ws, xbc = 0, 0, None, None
    if decode_rows < n:
        assert spans.dtype == torch.int32 and spans.is_contiguous() and spans.shape[1] == 4
        assert ring_slot.dtype == torch.int32 and ring_slot.is_contiguous() and tuple(ring_slot.shape) == (n, 2)
        num_spans = spans.shape[0]
        need = lib.infer_state_space_workspace_floats(elem, s.heads, s.vdim, s.state, num_spans, max_span)
        ws = torch.empty(need, dtype=torch.float32, device=proj.device) if need else None
        xbc = torch.empty((n - decode_rows, s.channels), dtype=proj.dtype, device=proj.device)
    y = torch.empty((n, s.inner), dtype=proj.dtype, device=proj.device)
    _require_gpu(proj, conv, ring, state, out)
    rc = lib.infer_state_space(
        elem, proj.data_ptr(), _rows(proj, max(z + s.inner, x + s.channels, dt + s.heads)), z, x, dt, s.heads, s.vdim, s.state, s.groups,
        s.taps, conv.data_ptr(), conv_bias.data_ptr(), dt_bias.data_ptr(), a_log.data_ptr(), d.data_ptr(), norm.data_ptr(), s.norm_parts,
        float(s.eps), ring.data_ptr(), state.data_ptr(), state.shape[0], _ptr(slots) if decode_rows else None, positions.data_ptr(),
        decode_rows, _ptr(spans) if num_spans else None, num_spans, max_span, _ptr(ring_slot) if num_spans else None, n, _ptr(xbc),
        y.data_ptr(), _ptr(ws), need, out.data_ptr(), _rows(out, s.inner), _stream_ptr(proj))
    _lib.check(rc, "state_space")


# ------------------------------------------------------------------ mixture of experts
@dataclass(frozen=True)
class MoeShape:
    """Sizes and constants of a router and its experts; ``identity`` entries behind the experts give the input itself.  Of ``groups``
    equal groups of entries the best ``keep`` are open to choice."""
    width: int
    ff: int
    experts: int
    top: int
    identity: int = 0
    groups: int = 1
    keep: int = 1
    scale: float = 1.0

    @property
    def ff_pad(self) -> int:
        return -(-self.ff // 8) * 8


def moe(s: MoeShape, h, router, correction, gate_up, down, counts) -> ExpertSum:
    """``h`` [tokens, width]; ``router`` [experts + identity, width], ``correction`` (float32) of the choice; ``gate_up``
    [experts, 2 * ff, width], ``down`` [experts, width, ff_pad] (zeros behind ff); ``counts`` [experts] int32 zeros."""
    n = h.shape[0]
    assert h.dtype == router.dtype == gate_up.dtype == down.dtype
    assert router.is_contiguous() and tuple(router.shape) == (s.experts + s.identity, s.width)
    assert gate_up.is_contiguous() and tuple(gate_up.shape) == (s.experts, 2 * s.ff, s.width)
    assert down.is_contiguous() and tuple(down.shape) == (s.experts, s.width, s.ff_pad)
    assert counts.dtype == torch.int32 and counts.is_contiguous() and counts.numel() == s.experts
    if correction is not None:
        _f32(correction, s.experts + s.identity)
    _require_gpu(h, router, gate_up, down, counts)
    lib, elem = _lib.load(), ELEM[h.dtype]
    layout = (ctypes.c_int64 * 3)()
    _lib.check(lib.infer_moe_layout(elem, n, s.width, s.ff_pad, s.experts, s.top, ctypes.addressof(layout)), "moe_layout")
    places_n, tiles_n, _ = layout
    ints = torch.empty(5 * places_n + 2 * tiles_n + s.experts + 1, dtype=torch.int32, device=h.device)
    ids, ranks, places, row_token, row_expert = (ints[i * places_n:(i + 1) * places_n] for i in range(5))
    tiles, offsets = ints[5 * places_n:5 * places_n + 2 * tiles_n], ints[5 * places_n + 2 * tiles_n:]
    weights = torch.empty((n, s.top), dtype=torch.float32, device=h.device)
    act = torch.empty((places_n, s.ff_pad), dtype=h.dtype, device=h.device)
    rows = torch.empty((places_n, s.width), dtype=h.dtype, device=h.device)
    rc = lib.infer_moe(
        elem, h.data_ptr(), _rows(h, s.width), router.data_ptr(), _ptr(correction), n, s.width, s.experts, s.identity, s.top, s.groups,
        s.keep, float(s.scale), gate_up.data_ptr(), down.data_ptr(), s.ff, s.ff_pad, counts.data_ptr(), ids.data_ptr(),
        weights.data_ptr(), ranks.data_ptr(), places.data_ptr(), row_token.data_ptr(), row_expert.data_ptr(), offsets.data_ptr(),
        tiles.data_ptr(), tiles_n, act.data_ptr(), rows.data_ptr(), places_n, _stream_ptr(h))
    _lib.check(rc, "moe")
    return ExpertSum(rows, places.view(n, s.top), weights, h)


# ------------------------------------------------------------------ linear attention with a constant decay
@lru_cache(maxsize=None)
def decay_layout(dim: int, vdim: int) -> tuple[int, int]:
    """(state rows, state columns) of a head."""
    out = (ctypes.c_int64 * 2)()
    _lib.check(_lib.load().infer_decay_layout(dim, vdim, ctypes.addressof(out)), "decay_layout")
    return tuple(out)


def decay_constants(decay, device) -> torch.Tensor:
    """[3, heads] float32: every decay rounded to float, what that leaves out, and its base-2 logarithm."""
    d = torch.tensor(decay, dtype=torch.float64)
    hi = d.float()
    return torch.stack((hi, (d - hi.double()).float(), torch.log2(d).clamp(min=-1e4).float())).contiguous().to(device)


class DecayShape:
    """Sizes and constants of a layer of linear attention with a constant decay per head."""

    def __init__(self, heads: int, dim: int, vdim: int, eps: float, silu: bool, rot_dims: int, scale: float, norm_per_head: bool,
                 gate_silu: bool):
        self.heads, self.dim, self.vdim, self.eps, self.silu, self.rot_dims = heads, dim, vdim, eps, silu, rot_dims
        self.scale, self.norm_per_head, self.gate_silu = scale, norm_per_head, gate_silu
        self.state_rows, self.state_cols = decay_layout(dim, vdim)


def decay_attention(s: DecayShape, proj, offsets, decay, table, norm, state, slots, positions, decode_rows: int, spans, max_span: int,
                    out) -> None:
    """``proj`` holds q, k, v and the gate logits at the columns ``offsets``.  Rows below ``decode_rows`` advance the state of
    ``slots[r]`` by one token (negative: padding), the others belong to ``spans`` [.., 4] (first row, tokens, slot, first
    position).  ``max_span`` is the number of tokens of the longest.  ``decay`` comes from
    ``decay_constants``."""
    n = proj.shape[0]
    q, k, v, g = offsets
    assert proj.dtype == out.dtype and out.shape[0] == n
    _f32(decay, 3, s.heads)
    _f32(state, state.shape[0], s.heads, s.state_rows, s.state_cols)
    if norm is not None:
        _f32(norm, s.heads * s.vdim)
    if s.rot_dims:
        assert table.dtype == torch.float32 and table.is_contiguous() and table.shape[1:] == (s.rot_dims // 2, 2)
    if decode_rows:
        assert slots.dtype == torch.int32 and slots.is_contiguous() and slots.numel() >= decode_rows
        assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() >= decode_rows
    lib, num_spans, ws, need = _lib.load(), 0, None, 0
    if decode_rows < n:
        assert spans.dtype == torch.int32 and spans.is_contiguous() and spans.shape[1] == 4
        num_spans = spans.shape[0]
        need = lib.infer_decay_workspace_floats(ELEM[proj.dtype], s.heads, s.dim, s.vdim, s.rot_dims, num_spans, max_span)
        ws = torch.empty(need, dtype=torch.float32, device=proj.device) if need else None
    _require_gpu(proj, decay, state, out)
    rc = lib.infer_decay_attention(
        ELEM[proj.dtype], proj.data_ptr(), _rows(proj, max(q + s.heads * s.dim, k + s.heads * s.dim, v + s.heads * s.vdim, g + s.heads * s.vdim)),
        q, k, v, g, s.heads, s.dim, s.vdim, decay.data_ptr(), int(s.silu), _ptr(table) if s.rot_dims else None, s.rot_dims,
        table.shape[0] if s.rot_dims else 1, float(s.scale), _ptr(norm), int(s.norm_per_head), int(s.gate_silu), float(s.eps),
        state.data_ptr(), state.shape[0], _ptr(slots), _ptr(positions), decode_rows, _ptr(spans) if num_spans else None, num_spans, max_span, n,
        _ptr(ws), need, out.data_ptr(), _rows(out, s.heads * s.vdim), _stream_ptr(proj))
    _lib.check(rc, "decay_attention")


# ------------------------------------------------------------------ gated delta rule
@lru_cache(maxsize=None)
def delta_layout(dim: int, vdim: int) -> tuple[int, int, int, int]:
    """(state rows, state columns, floats of a chunk record, tokens per chunk) of a head."""
    out = (ctypes.c_int64 * 4)()
    _lib.check(_lib.load().infer_delta_layout(dim, vdim, ctypes.addressof(out)), "delta_layout")
    return tuple(out)


class DeltaShape:
    """Sizes and constants of a delta-rule layer, shared by its two entry points."""

    def __init__(self, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, eps: float):
        assert heads % kv_heads == 0
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps, self.eps = heads, kv_heads, dim, vdim, taps, eps
        self.channels = 2 * kv_heads * dim + heads * vdim
        self.state_rows, self.state_cols, self.record, self.chunk = delta_layout(dim, vdim)


def _delta_common(s: DeltaShape, proj, beta_off, decay, gate, conv, a_log, dt_bias, norm, ring, state, out):
    assert proj.dtype == decay.dtype == gate.dtype == ring.dtype == out.dtype
    n = proj.shape[0]
    assert decay.shape[0] == gate.shape[0] == out.shape[0] == n
    slots = state.shape[0]
    _f32(conv, s.channels, s.taps)
    _f32(a_log, s.heads)
    _f32(dt_bias, s.heads * s.dim)
    _f32(norm, s.vdim)
    _f32(state, slots, s.heads, s.state_rows, s.state_cols)
    assert ring.is_contiguous() and tuple(ring.shape) == (slots, s.taps, s.channels)
    _require_gpu(proj, decay, gate, conv, a_log, dt_bias, norm, ring, state, out)
    return [ELEM[proj.dtype], proj.data_ptr(), _rows(proj, beta_off + s.heads), beta_off, decay.data_ptr(),
            _rows(decay, s.heads * s.dim), gate.data_ptr(), _rows(gate, s.heads * s.vdim), conv.data_ptr(), a_log.data_ptr(),
            dt_bias.data_ptr(), norm.data_ptr(), ring.data_ptr(), state.data_ptr(), slots, s.heads, s.kv_heads, s.dim, s.vdim,
            s.taps, float(s.eps)]


def delta_step(s: DeltaShape, proj, beta_off, decay, gate, conv, a_log, dt_bias, norm, ring, state, slots, positions, out) -> None:
    """One token per sequence: row r of the inputs advances the state of slot ``slots[r]`` (negative: padding)."""
    n = proj.shape[0]
    args = _delta_common(s, proj, beta_off, decay, gate, conv, a_log, dt_bias, norm, ring, state, out)
    assert slots.dtype == torch.int32 and slots.is_contiguous() and slots.numel() == n
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == n
    rc = _lib.load().infer_delta_step(*args, slots.data_ptr(), positions.data_ptr(), out.data_ptr(), _rows(out, s.heads * s.vdim),
                                      n, _stream_ptr(proj))
    _lib.check(rc, "delta_step")


def delta_chunks(s: DeltaShape, proj, beta_off, decay, gate, conv, a_log, dt_bias, norm, ring, state, portions, chunks, ring_slot,
                 positions, row0: int, out) -> None:
    """Prompt portions: batch rows ``row0`` and up.  ``portions`` [.., 4] and ``chunks`` [.., 6] are the int32
    descriptors of ``infer_kv.h``; ``ring_slot`` and ``positions`` are indexed by batch row."""
    n = proj.shape[0]
    args = _delta_common(s, proj, beta_off, decay, gate, conv, a_log, dt_bias, norm, ring, state, out)
    assert portions.dtype == torch.int32 and portions.is_contiguous() and portions.shape[1] == 4
    assert chunks.dtype == torch.int32 and chunks.is_contiguous() and chunks.shape[1] == 6
    assert ring_slot.dtype == torch.int32 and ring_slot.is_contiguous() and tuple(ring_slot.shape) == (n, 2)
    assert positions.dtype == torch.int64 and positions.is_contiguous() and positions.numel() == n
    records = torch.empty(chunks.shape[0] * s.heads * s.record, dtype=torch.float32, device=proj.device)
    o = torch.empty(n * s.heads * s.state_cols, dtype=torch.float32, device=proj.device)
    rc = _lib.load().infer_delta_chunks(
        *args, portions.data_ptr(), portions.shape[0], chunks.data_ptr(), chunks.shape[0], records.data_ptr(), o.data_ptr(),
        ring_slot.data_ptr(), positions.data_ptr(), out.data_ptr(), _rows(out, s.heads * s.vdim), row0, n - row0, _stream_ptr(proj))
    _lib.check(rc, "delta_chunks")
