"""Latent attention: keys and values are linear in one compressed row per token, which is all that is cached.

``LatentAttention`` holds the weights; the cache pages are an argument, so that several layers can run on the
same weights with pages of their own.  Two forms of the same attention:

* rows: the query goes into the latent space (``W_uk^T q`` per head), attends over the cached rows themselves
  and the weighted latent comes out through ``W_uv``.  Decoded tokens, tokens of short portions, float32.
* dense: the latents of the whole sequence are expanded to keys and values once, for portions long enough to
  pay for it (3-4 times fewer operations per query-key pair)."""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from . import hybrid_ops
from .cache import LatentPages
from .context import get_context
from .layers import Linear, PackedLinear, yarn_rotary_table


def _up(n: int, to: int) -> int:
    return -(-n // to) * to


class LatentAttention(nn.Module):

    def __init__(self, hidden_size: int, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, scale: float,
                 rot: dict, eps: float, dtype: torch.dtype):
        """``rot``: ``base``, ``dims`` (rotated entries at the front of the rotated part) and optionally ``scaling``."""
        super().__init__()
        self.heads, self.dim, self.rot_dim, self.vdim, self.rank = heads, dim, rot_dim, vdim, kv_rank
        self.scale, self.rot, self.eps, self.dtype = scale, rot, eps, dtype
        self.rank_pad = _up(kv_rank, 32)
        self.row = self.rank_pad + _up(rot_dim, 32)
        self.in_proj = PackedLinear(hidden_size, {"q": heads * (dim + rot_dim), "dkv": kv_rank + rot_dim, "g": heads}, dtype)
        self.latent_norm = nn.Parameter(torch.ones(kv_rank), requires_grad=False)
        self.k_up = nn.Parameter(torch.empty(heads * dim, kv_rank, dtype=dtype), requires_grad=False)
        self.v_up = nn.Parameter(torch.empty(heads * vdim, kv_rank, dtype=dtype), requires_grad=False)
        self.o_proj = Linear(heads * vdim, hidden_size, dtype=dtype)

    def cache_spec(self) -> LatentPages:
        return LatentPages(self.row, self.dtype)

    def finish_loading(self, max_position: int) -> None:
        """Forms of the up-projections that the kernels read, and the table of rotations."""
        device = self.k_up.device
        h, d, v, r, rp = self.heads, self.dim, self.vdim, self.rank, self.rank_pad
        absorb = torch.zeros(h, rp, _up(d, 32), dtype=self.dtype, device=device)       # [head][latent][dim]
        absorb[:, :r, :d] = self.k_up.data.view(h, d, r).transpose(1, 2)
        out = torch.zeros(h, _up(v, 16), rp, dtype=self.dtype, device=device)           # [head][value][latent]
        out[:, :v, :r] = self.v_up.data.view(h, v, r)
        self.absorb, self.out_up = absorb, out
        # the dense kernel reads a head's part of a row in 16-byte pieces
        self.dense = self.dtype == torch.bfloat16 and hybrid_ops.latent_prefill_supported(d, self.rot_dim, v)
        self.expand = F.pad(torch.cat((self.k_up.data, self.v_up.data)), (0, rp - r)).contiguous() if self.dense else None
        self.table = yarn_rotary_table(self.rot["dims"], max_position, self.rot["base"], self.rot.get("scaling"), device)

    def forward(self, h: torch.Tensor, pages: torch.Tensor) -> torch.Tensor:
        plan = get_context().step
        n, heads = h.shape[0], self.heads
        proj = self.in_proj(h)
        gate = self.in_proj.piece(proj, "g")
        split = plan.dense_row if self.dense else n            # rows from here on attend over dense keys
        out = torch.empty((n, heads * self.vdim), dtype=h.dtype, device=h.device)
        qx = torch.empty((split, heads, self.row), dtype=h.dtype, device=h.device)
        hybrid_ops.latent_front(proj, heads, self.dim, self.rot_dim, self.rot["dims"], self.in_proj.offset["dkv"], self.rank,
                                self.latent_norm, self.eps, self.table, plan.positions, plan.slot_mapping, pages,
                                self.rank_pad, qx, split)
        q = proj[:, :heads * (self.dim + self.rot_dim)]
        if split > 0:
            q3 = q[:split].unflatten(1, (heads, self.dim + self.rot_dim))
            hybrid_ops.head_matmul(q3, self.absorb, qx, self.rank_pad, self.dim)
            o = hybrid_ops.latent_attention(qx, pages, plan.block_tables, plan.row_ctx[:split], self.scale, self.rank_pad,
                                            row_seq=None if plan.row_seq is None else plan.row_seq[:split],
                                            max_keys=plan.max_keys)
            hybrid_ops.head_matmul(o, self.out_up, out[:split].unflatten(1, (heads, self.vdim)), self.vdim, self.rank_pad,
                                   gate=gate[:split])
        if split < n:
            rows = hybrid_ops.latent_gather(pages, plan.block_tables, plan.dense_seqs, plan.dense_cu_k, plan.dense_keys,
                                            plan.dense_max_k)
            kv = F.linear(rows[:, :self.rank_pad], self.expand)
            hybrid_ops.latent_prefill(q[split:], kv[:, :heads * self.dim], rows[:, self.rank_pad:self.rank_pad + self.rot_dim],
                                      kv[:, heads * self.dim:], gate[split:], out[split:], plan.dense_cu_q, plan.dense_cu_k,
                                      plan.dense_max_q, heads, self.dim, self.rot_dim, self.vdim, self.scale)
        return self.o_proj(out, defer=True)
