"""Attention whose queries see the keys of a chunk or of a window, over pages of ``[value | key]`` rows: a part of a ``Mixer``.

Everything that tells one such attention from another is a parameter: biases of the projections, norms per head, rotary positions,
a bias of the scores that grows with the distance, a softmax sink, a gate per head, two maps (the difference of two attentions over
the same values).  Decoded tokens, tokens of short portions and float32 run row by row against the pages; portions long
enough to pay for it gather the keys of their sequence once and run as dense tiles."""
from __future__ import annotations

import math

import torch
from torch import nn

from . import hybrid_ops
from .cache import GroupedPages
from .context import get_context
from .layers import banded_rotary_table


def _vector(size: int, value: float = 0.0) -> nn.Parameter:
    return nn.Parameter(torch.full((size,), value), requires_grad=False)


class MaskedAttention(nn.Module):
    dense_pieces = ()

    def __init__(self, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, eps: float, dtype: torch.dtype, *,
                 mask: str | None = None, mask_size: int = 1, rot: dict | None = None, bias: bool = False, head_norm: bool = False,
                 distance_bias: bool = False, sink: bool = False, gate: bool = False, diff: float | None = None, out_scale: float = 1.0):
        """``rot``: ``base``, ``dims`` (rotated entries at the front of a head; entry i turns with entry i + dims / 2) and optionally
        ``scaling``.  ``diff``: two maps, and the constant of their difference."""
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads cannot share {kv_heads} key heads")
        if mask is not None and mask_size < 1:
            raise ValueError(f"a mask of {mask_size} tokens shows nothing")
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.rot, self.dtype, self.diff = rot, dtype, diff
        self.maps = 1 if diff is None else 2
        self.constants = dict(scale=scale, maps=self.maps, mask=mask, mask_size=mask_size, distance_bias=distance_bias, eps=eps,
                              rot_dims=rot["dims"] if rot else 0, out_scale=out_scale if diff is None else (1.0 - diff) * out_scale)
        self.biased_pieces = ("q", "k", "v") if bias else ()
        self.has_gate = gate
        self.q_norm, self.k_norm = (_vector(dim, 1.0), _vector(dim, 1.0)) if head_norm else (None, None)
        self.sink = _vector(heads) if sink else None
        if diff is not None:
            self.lq1, self.lk1, self.lq2, self.lk2 = (_vector(dim) for _ in range(4))
        self.out_size = heads * vdim
        self.shape = self._shape(0.0)

    def _shape(self, lam: float) -> hybrid_ops.MaskedShape:
        return hybrid_ops.MaskedShape(self.heads, self.kv_heads, self.dim, self.vdim, lam=lam, **self.constants)

    def pieces(self) -> dict[str, int]:
        pieces = {"q": self.heads * self.maps * self.dim, "k": self.kv_heads * self.maps * self.dim, "v": self.kv_heads * self.vdim}
        return pieces | ({"g": self.heads} if self.has_gate else {})

    def cache_spec(self) -> GroupedPages:
        return GroupedPages(self.kv_heads, self.shape.vdim_pad + self.shape.key_pad, self.dtype)

    def finish_loading(self, max_position: int) -> None:
        lam = 0.0
        if self.diff is not None:
            first, second = (float((a.double() * b.double()).sum()) for a, b in ((self.lq1, self.lk1), (self.lq2, self.lk2)))
            lam = math.exp(first) - math.exp(second) + self.diff
        self.shape = self._shape(lam)
        self.dense = self.dtype == torch.bfloat16 and hybrid_ops.masked_prefill_supported(self.shape)
        self.table = None
        if self.rot:
            device = torch.device("cuda", torch.cuda.current_device())
            self.table = banded_rotary_table(self.rot["dims"], max_position, self.rot["base"], self.rot.get("scaling"), device)

    def forward(self, proj: torch.Tensor, offset: dict, bias, pages: torch.Tensor, out: torch.Tensor) -> None:
        plan, s = get_context().step, self.shape
        n = proj.shape[0]
        split = plan.dense_row if self.dense else n            # rows from here on attend over dense keys
        qx = torch.empty((split, s.heads * s.maps, s.key_pad), dtype=proj.dtype, device=proj.device)
        hybrid_ops.head_front(s, proj, [offset[name] for name in "qkv"], bias, self.q_norm, self.k_norm, self.table, plan.positions,
                              plan.slot_mapping, pages, qx, split)
        gate = proj[:, offset["g"]:offset["g"] + s.heads] if self.has_gate else None
        if split > 0:
            hybrid_ops.masked_attention(s, qx, pages, plan.block_tables, plan.row_ctx[:split], out[:split], self.sink,
                                        gate[:split] if gate is not None else None,
                                        row_seq=None if plan.row_seq is None else plan.row_seq[:split], max_keys=plan.max_keys)
        if split < n:
            rows = hybrid_ops.masked_gather(s, pages, plan.block_tables, plan.dense_seqs, plan.dense_cu_q, plan.dense_cu_k,
                                            plan.dense_keys, plan.dense_max_k)
            hybrid_ops.masked_prefill(s, proj[split:, offset["q"]:], rows, out[split:], plan.dense_cu_q, plan.dense_cu_k, plan.dense_max_q,
                                      self.sink, gate[split:] if gate is not None else None)
