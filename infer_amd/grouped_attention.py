"""Grouped attention with a softmax sink and an output gate per head, over pages of ``[value | key]`` rows.

``GroupedAttention`` holds the weights; the pages are an argument, and a layer without keys of its own
(``own_keys=False``) attends over the pages that an earlier layer has written in the same step.  Decoded tokens, tokens of
short portions and float32 run row by row against the pages; portions long enough to pay for it gather the keys of
their sequence once and run as dense tiles."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import GroupedPages
from .context import get_context
from .layers import Linear, PackedBias, PackedLinear, yarn_rotary_table


def _up(n: int, to: int) -> int:
    return -(-n // to) * to


class GroupedAttention(nn.Module):

    def __init__(self, hidden_size: int, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, rot: dict, eps: float,
                 dtype: torch.dtype, own_keys: bool = True):
        """``rot``: ``base``, ``dims`` (rotated entries at the front of a head) and optionally ``scaling``."""
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads cannot share {kv_heads} key heads")
        self.heads, self.kv_heads, self.dim, self.vdim = heads, kv_heads, dim, vdim
        self.scale, self.rot, self.eps, self.dtype, self.own_keys = scale, rot, eps, dtype, own_keys
        self.dim_pad, self.vdim_pad = _up(dim, 32), _up(vdim, 32)
        keys = {"k": kv_heads * dim, "v": kv_heads * vdim} if own_keys else {}
        self.in_proj = PackedLinear(hidden_size, {"q": heads * dim, **keys, "g": heads}, dtype)
        self.bias = PackedBias(self.in_proj, ("q", *keys))
        self.q_norm = nn.Parameter(torch.ones(heads * dim), requires_grad=False)
        self.k_norm = nn.Parameter(torch.ones(kv_heads * dim), requires_grad=False) if own_keys else None
        self.sink = nn.Parameter(torch.zeros(heads), requires_grad=False)
        self.o_proj = Linear(heads * vdim, hidden_size, dtype=dtype)

    def cache_spec(self) -> GroupedPages:
        return GroupedPages(self.kv_heads, self.vdim_pad + self.dim_pad, self.dtype)

    def finish_loading(self, max_position: int) -> None:
        self.dense = self.dtype == torch.bfloat16 and hybrid_ops.grouped_prefill_supported(self.dim, self.vdim)
        self.table = yarn_rotary_table(self.rot["dims"], max_position, self.rot["base"], self.rot.get("scaling"), self.sink.device)

    def forward(self, h: torch.Tensor, pages: torch.Tensor) -> torch.Tensor:
        plan = get_context().step
        n, heads = h.shape[0], self.heads
        proj = self.in_proj(h)
        gate = self.in_proj.piece(proj, "g")
        split = plan.dense_row if self.dense else n            # rows from here on attend over dense keys
        out = torch.empty((n, heads * self.vdim), dtype=h.dtype, device=h.device)
        qx = torch.empty((split, heads, self.dim_pad), dtype=h.dtype, device=h.device)
        offset = self.in_proj.offset
        hybrid_ops.grouped_front(proj, heads, self.kv_heads if self.own_keys else 0, self.dim, self.vdim, offset.get("k", 0),
                                 offset.get("v", 0), self.bias.weight, self.q_norm, self.k_norm, self.eps, self.table,
                                 self.rot["dims"], plan.positions, plan.slot_mapping, pages, self.dim_pad, self.vdim_pad, qx, split)
        if split > 0:
            hybrid_ops.grouped_attention(qx, pages, plan.block_tables, plan.row_ctx[:split], self.scale, self.vdim, out[:split],
                                         self.sink, gate[:split], row_seq=None if plan.row_seq is None else plan.row_seq[:split],
                                         max_keys=plan.max_keys)
        if split < n:
            rows = hybrid_ops.grouped_gather(pages, plan.block_tables, plan.dense_seqs, plan.dense_cu_k, plan.dense_keys,
                                             plan.dense_max_k)
            hybrid_ops.grouped_prefill(proj[split:], rows[:, :, self.vdim_pad:], rows[:, :, :self.vdim_pad], self.sink, gate[split:],
                                       out[split:], plan.dense_cu_q, plan.dense_cu_k, plan.dense_max_q, heads, self.dim, self.vdim,
                                       self.scale)
        return self.o_proj(out, defer=True)
