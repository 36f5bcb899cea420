"""Mixture of experts: a router that chooses inside the best groups, identity experts, a shared expert.

The weighted sum of a token's experts is not taken here but by the kernel of the residual sum (``hybrid_ops.ExpertSum``)."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .layers import GatedMLP


class ExpertMatrices(nn.Module):
    """Equal matrices of all experts in one tensor ``[experts, rows * parts, columns]``, loaded piece by piece; shard (expert, part)."""

    def __init__(self, experts: int, parts: int, rows: int, columns: int, pad_columns: int, dtype: torch.dtype):
        super().__init__()
        self.rows, self.columns = rows, columns
        self.sizes = {(e, p): rows for e in range(experts) for p in range(parts)}
        self.weight = nn.Parameter(torch.zeros(experts, parts * rows, pad_columns, dtype=dtype), requires_grad=False)

    def weight_loader(self, param: nn.Parameter, loaded_weight: torch.Tensor, shard_id: tuple[int, int]):
        expert, part = shard_id
        piece = param.data[expert, part * self.rows:(part + 1) * self.rows, :self.columns]
        if piece.shape != loaded_weight.shape:
            raise ValueError(f"expert {expert}: {tuple(loaded_weight.shape)} does not fit {tuple(piece.shape)}")
        piece.copy_(loaded_weight)


class MixtureOfExperts(nn.Module):

    def __init__(self, hidden_size: int, ff: int, experts: int, top: int, dtype: torch.dtype, *, identity: int = 0, groups: int = 1,
                 keep: int = 1, scale: float = 1.0, shared_ff: int | None = None):
        super().__init__()
        every = experts + identity
        if every % groups or not 1 <= keep <= groups or keep * (every // groups) < top:
            raise ValueError(f"{top} of {every} experts cannot be chosen from {keep} of {groups} groups")
        self.shape = s = hybrid_ops.MoeShape(hidden_size, ff, experts, top, identity, groups, keep, scale)
        self.router = nn.Parameter(torch.empty(every, hidden_size, dtype=dtype), requires_grad=False)
        self.correction = nn.Parameter(torch.zeros(every), requires_grad=False)
        self.gate_up = ExpertMatrices(experts, 2, ff, hidden_size, hidden_size, dtype)
        self.down = ExpertMatrices(experts, 1, hidden_size, ff, s.ff_pad, dtype)
        self.shared = GatedMLP(hidden_size, shared_ff, dtype, act="silu") if shared_ff is not None else None
        self.register_buffer("counts", torch.zeros(experts, dtype=torch.int32), persistent=False)   # scratch, zero between steps

    def forward(self, h: torch.Tensor) -> hybrid_ops.ExpertSum:
        out = hybrid_ops.moe(self.shape, h, self.router, self.correction, self.gate_up.weight, self.down.weight, self.counts)
        if self.shared is not None:
            out.shared = self.shared(h)               # last: an unreduced product must be consumed before the next one
        return out
