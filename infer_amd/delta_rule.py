"""Gated delta rule with a decay per key channel: a recurrent layer with a ``[dim, vdim]`` state per head.

As with ``LatentAttention``, the module holds the weights and the state is an argument.  Decoded tokens run
through one fused kernel, prompt portions through the chunked kernels; both read and write the same state."""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from . import hybrid_ops
from .cache import StateSlots
from .context import get_context
from .layers import Linear, PackedLinear


class ChannelDelta(nn.Module):

    def __init__(self, hidden_size: int, heads: int, kv_heads: int, dim: int, vdim: int, conv: int, decay_rank: int,
                 gate_rank: int, eps: float, dtype: torch.dtype):
        super().__init__()
        self.shape = hybrid_ops.DeltaShape(heads, kv_heads, dim, vdim, conv, eps)
        self.dtype = dtype
        # q, k and v come without gaps: the convolution's channels are the first columns of a row
        qkv = {"q": kv_heads * dim, "k": kv_heads * dim, "v": heads * vdim}
        self.in_proj = PackedLinear(hidden_size, qkv | {"b": heads, "a1": decay_rank, "g1": gate_rank}, dtype, dense=("q", "k"))
        self.decay_up = Linear(decay_rank, heads * dim, dtype=dtype)
        self.gate_up = Linear(gate_rank, heads * vdim, dtype=dtype)
        self.conv = ConvTaps(qkv, conv)
        self.a_log = nn.Parameter(torch.zeros(heads), requires_grad=False)
        self.dt_bias = nn.Parameter(torch.zeros(heads * dim), requires_grad=False)
        self.out_norm = nn.Parameter(torch.ones(vdim), requires_grad=False)
        self.o_proj = Linear(heads * vdim, hidden_size, dtype=dtype)

    def cache_spec(self) -> StateSlots:
        s = self.shape
        return StateSlots(state=((s.heads, s.state_rows, s.state_cols), torch.float32), ring=((s.taps, s.channels), self.dtype))

    def finish_loading(self, max_position: int) -> None:
        pass

    def forward(self, h: torch.Tensor, cache: dict) -> torch.Tensor:
        plan = get_context().step
        s, d = self.shape, plan.decode_rows
        proj = self.in_proj(h)
        decay = F.linear(self.in_proj.piece(proj, "a1"), self.decay_up.weight)
        gate = F.linear(self.in_proj.piece(proj, "g1"), self.gate_up.weight)
        out = torch.empty((h.shape[0], s.heads * s.vdim), dtype=h.dtype, device=h.device)
        weights = (self.conv.weight, self.a_log, self.dt_bias, self.out_norm, cache["ring"], cache["state"])
        beta = self.in_proj.offset["b"]
        if d > 0:
            hybrid_ops.delta_step(s, proj[:d], beta, decay[:d], gate[:d], *weights, plan.state_slots, plan.positions[:d], out[:d])
        if d < h.shape[0]:
            hybrid_ops.delta_chunks(s, proj, beta, decay, gate, *weights, plan.portions, plan.chunks, plan.ring_slot,
                                    plan.positions, d, out)
        return self.o_proj(out, defer=True)


class ConvTaps(nn.Module):
    """Taps of a causal convolution per channel, ``[channels, taps]`` float32, loaded in named runs of channels."""

    def __init__(self, runs: dict[str, int], taps: int):
        super().__init__()
        self.sizes = dict(runs)
        self.weight = nn.Parameter(torch.zeros(sum(runs.values()), taps), requires_grad=False)

    def weight_loader(self, param: nn.Parameter, loaded_weight: torch.Tensor, shard_id: str):
        names = list(self.sizes)
        start = sum(self.sizes[n] for n in names[:names.index(shard_id)])
        rows = param.data.narrow(0, start, self.sizes[shard_id])
        if rows.shape != loaded_weight.shape:
            raise ValueError(f"convolution {shard_id!r}: {tuple(loaded_weight.shape)} does not fit {tuple(rows.shape)}")
        rows.copy_(loaded_weight)
