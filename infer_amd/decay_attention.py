"""Linear attention with a constant decay per head: a recurrent layer with a ``[dim, vdim]`` float32 state per head and
neither softmax nor denominator.

The module holds the weights and the state is an argument.  What stands in front of and behind the recurrence are
parameters: silu on q, k and v or a rotary embedding of q and k; a norm over each head or over all heads together,
with or without a weight; a sigmoid or silu output gate."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import StateSlots
from .context import get_context
from .layers import Linear, PackedLinear, yarn_rotary_table


class DecayAttention(nn.Module):

    def __init__(self, hidden_size: int, heads: int, dim: int, vdim: int, decay: list[float], eps: float, dtype: torch.dtype, *,
                 silu: bool = False, rot: dict | None = None, scale: float = 1.0, norm_per_head: bool = False,
                 norm_weight: bool = True, gate_silu: bool = False):
        """``rot``: ``base`` and ``dims`` (rotated entries at the front of a head; entry i turns with entry i + dims / 2)."""
        super().__init__()
        if len(decay) != heads:
            raise ValueError(f"{len(decay)} decays for {heads} heads")
        self.rot, self.decay_values, self.dtype = rot, decay, dtype
        self.shape = hybrid_ops.DecayShape(heads, dim, vdim, eps, silu, rot["dims"] if rot else 0, scale, norm_per_head, gate_silu)
        self.in_proj = PackedLinear(hidden_size, {"q": heads * dim, "k": heads * dim, "v": heads * vdim, "g": heads * vdim}, dtype)
        self.out_norm = nn.Parameter(torch.ones(heads * vdim), requires_grad=False) if norm_weight else None
        self.o_proj = Linear(heads * vdim, hidden_size, dtype=dtype)

    def cache_spec(self) -> StateSlots:
        s = self.shape
        return StateSlots(state=((s.heads, s.state_rows, s.state_cols), torch.float32))

    def finish_loading(self, max_position: int) -> None:
        device = self.o_proj.weight.device
        self.decay = hybrid_ops.decay_constants(self.decay_values, device)
        self.table = yarn_rotary_table(self.rot["dims"], max_position, self.rot["base"], None, device) if self.rot else None

    def forward(self, h: torch.Tensor, cache: dict) -> torch.Tensor:
        plan, s = get_context().step, self.shape
        proj = self.in_proj(h)
        out = torch.empty((h.shape[0], s.heads * s.vdim), dtype=h.dtype, device=h.device)
        offset = self.in_proj.offset
        hybrid_ops.decay_attention(s, proj, [offset[name] for name in "qkvg"], self.decay, self.table, self.out_norm, cache["state"],
                                   plan.state_slots, plan.positions, plan.decode_rows, plan.spans, plan.max_span, out)
        return self.o_proj(out, defer=True)
