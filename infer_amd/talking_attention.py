"""Attention whose heads mix their softmax weights before these meet the values (talking heads), over pages of tiles:
a part of a ``Mixer``.

Queries and keys are divided by their root mean square per head, optionally values too; queries may have a temperature that grows with
the position; every softmax denominator has a one added to it.  Decoded tokens, tokens of short portions and float32 run row by row with their
scores in memory; long portions run in tiles that compute the scores twice instead."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import TilePages
from .context import get_context


class TalkingAttention(nn.Module):
    dense_pieces = ()
    biased_pieces = ()

    def __init__(self, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, eps: float, dtype: torch.dtype, *,
                 norm_values: bool = True, temperature: dict | None = None, out_scale: float = 1.0):
        """``temperature``: ``coef`` and ``every``."""
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} query heads cannot share {kv_heads} key heads")
        named = {}
        if temperature:
            if temperature["every"] <= 0:
                raise ValueError(f"a temperature cannot change every {temperature['every']} tokens")
            named = dict(temp_coef=temperature["coef"], temp_every=temperature["every"])
        self.shape = hybrid_ops.TalkShape(heads, kv_heads, dim, vdim, scale, eps, norm_values, out_scale=out_scale, **named)
        self.dtype, self.out_size = dtype, heads * vdim
        self.talk = nn.Parameter(torch.eye(heads, dtype=dtype), requires_grad=False)

    def pieces(self) -> dict[str, int]:
        s = self.shape
        return {"q": s.heads * s.dim, "k": s.kv_heads * s.dim, "v": s.kv_heads * s.vdim}

    def cache_spec(self) -> TilePages:
        return TilePages(self.shape.kv_heads, self.shape.key_pad, self.shape.vdim_pad, self.dtype)

    def finish_loading(self, max_position: int) -> None:
        pass

    def forward(self, proj: torch.Tensor, offset: dict, bias, pages: dict, out: torch.Tensor) -> None:
        plan, s, keys, values = get_context().step, self.shape, pages["keys"], pages["values"]
        n = proj.shape[0]
        dense = self.dtype == torch.bfloat16 and hybrid_ops.talking_prefill_supported(s)
        split = plan.dense_row if dense else n                 # rows from here on belong to long portions
        qx = torch.empty((split, s.heads, s.key_pad), dtype=proj.dtype, device=proj.device)
        hybrid_ops.unit_head_front(s, proj, [offset[name] for name in "qkv"], plan.positions, plan.slot_mapping, keys, values, qx, split)
        if split > 0:
            hybrid_ops.talking_attention(s, qx, keys, values, self.talk, plan.block_tables, plan.row_ctx[:split], out[:split],
                                         row_seq=None if plan.row_seq is None else plan.row_seq[:split], max_keys=plan.max_keys)
        if split < n:
            hybrid_ops.talking_prefill(s, proj[split:, offset["q"]:], keys, values, self.talk, plan.block_tables, plan.dense_seqs, plan.dense_cu_q,
                                       plan.dense_cu_k, plan.dense_max_q, plan.dense_max_k, out[split:], max_score=s.max_score(plan.max_keys))
