"""Linear attention with a constant decay per head: a recurrent layer with a ``[dim, vdim]`` float32 state per head and
neither softmax nor denominator.

``DecayHeads`` is a part of a ``Mixer``, ``DecayAttention`` a layer of its own with its projections; the state is an
argument.  What stands in front of and behind the recurrence are parameters: silu on q, k and v or a rotary embedding of
q and k; a norm over each head or over all heads together, with or without a weight; a sigmoid or silu output gate."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import StateSlots
from .context import get_context
from .layers import Linear, PackedLinear, yarn_rotary_table


class DecayHeads(nn.Module):
    dense_pieces = ()
    biased_pieces = ()

    def __init__(self, heads: int, dim: int, vdim: int, decay: list[float], eps: float, dtype: torch.dtype, *, silu: bool = False,
                 rot: dict | None = None, scale: float = 1.0, norm_per_head: bool = False, norm_weight: bool = True, gate_silu: bool = False,
                 out_scale: float = 1.0):
        """``rot``: ``base`` and ``dims`` (rotated entries at the front of a head; entry i turns with entry i + dims / 2)."""
        super().__init__()
        if len(decay) != heads:
            raise ValueError(f"{len(decay)} decays for {heads} heads")
        self.rot, self.decay_values, self.dtype, self.out_scale, self.out_size = rot, decay, dtype, out_scale, heads * vdim
        self.shape = hybrid_ops.DecayShape(heads, dim, vdim, eps, silu, rot["dims"] if rot else 0, scale, norm_per_head, gate_silu)
        self.out_norm = nn.Parameter(torch.ones(heads * vdim), requires_grad=False) if norm_weight else None

    def pieces(self) -> dict[str, int]:
        s = self.shape
        return {"q": s.heads * s.dim, "k": s.heads * s.dim, "v": s.heads * s.vdim, "g": s.heads * s.vdim}

    def cache_spec(self) -> StateSlots:
        s = self.shape
        return StateSlots(state=((s.heads, s.state_rows, s.state_cols), torch.float32))

    def finish_loading(self, max_position: int) -> None:
        device = torch.device("cuda", torch.cuda.current_device())
        self.decay = hybrid_ops.decay_constants(self.decay_values, device)
        self.table = yarn_rotary_table(self.rot["dims"], max_position, self.rot["base"], None, device) if self.rot else None
        self.gain = self.out_norm.data if self.out_norm is not None else None       # behind the norm
        if self.out_scale != 1.0:
            self.gain = (self.gain if self.gain is not None else torch.ones(self.out_size, device=device)) * self.out_scale

    def forward(self, proj: torch.Tensor, offset: dict, bias, cache: dict, out: torch.Tensor) -> None:
        plan = get_context().step
        hybrid_ops.decay_attention(self.shape, proj, [offset[name] for name in "qkvg"], self.decay, self.table, self.gain, cache["state"],
                                   plan.state_slots, plan.positions, plan.decode_rows, plan.spans, plan.max_span, out)


class DecayAttention(DecayHeads):

    def __init__(self, hidden_size: int, heads: int, dim: int, vdim: int, decay: list[float], eps: float, dtype: torch.dtype, **named):
        super().__init__(heads, dim, vdim, decay, eps, dtype, **named)
        self.in_proj = PackedLinear(hidden_size, self.pieces(), dtype)
        self.o_proj = Linear(self.out_size, hidden_size, dtype=dtype)

    def forward(self, h: torch.Tensor, cache: dict) -> torch.Tensor:
        out = torch.empty((h.shape[0], self.out_size), dtype=h.dtype, device=h.device)
        super().forward(self.in_proj(h), self.in_proj.offset, None, cache, out)
        return self.o_proj(out, defer=True)
