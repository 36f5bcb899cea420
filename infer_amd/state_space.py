"""Selective state space (Mamba-2) with a ``[state, vdim]`` float32 state per head: a part of a ``Mixer``.

Decoded tokens run through one fused kernel, prompt portions through the chunked kernels; both read and write the same state
and the same ring of convolution inputs."""
from __future__ import annotations

import torch
from torch import nn

from . import hybrid_ops
from .cache import StateSlots
from .context import get_context


def _zeros(*shape: int) -> nn.Parameter:
    return nn.Parameter(torch.zeros(*shape), requires_grad=False)


class StateSpace(nn.Module):
    dense_pieces = ()
    biased_pieces = ()

    def __init__(self, heads: int, vdim: int, state: int, groups: int, conv: int, norm_parts: int, eps: float, dtype: torch.dtype, *,
                 out_scale: float = 1.0):
        super().__init__()
        if heads % groups or heads * vdim % norm_parts:
            raise ValueError(f"{heads} heads of {vdim} do not divide into {groups} groups and {norm_parts} parts of a norm")
        self.shape = s = hybrid_ops.StateSpaceShape(heads, vdim, state, groups, conv, norm_parts, eps)
        self.dtype, self.out_scale, self.out_size = dtype, out_scale, s.inner
        self.conv, self.conv_bias = _zeros(s.channels, conv), _zeros(s.channels)
        self.dt_bias, self.a_log, self.d = _zeros(heads), _zeros(heads), _zeros(heads)
        self.out_norm = nn.Parameter(torch.ones(s.inner), requires_grad=False)

    def pieces(self) -> dict[str, int]:
        return {"in": self.shape.inner + self.shape.channels + self.shape.heads}          # [z | x | B | C | dt]

    def cache_spec(self) -> StateSlots:
        s = self.shape
        return StateSlots(state=((s.heads, s.state, s.vdim), torch.float32), ring=((s.taps, s.channels), self.dtype))

    def finish_loading(self, max_position: int) -> None:
        self.gain = (self.out_norm.data * self.out_scale).contiguous()

    def forward(self, proj: torch.Tensor, offset: dict, bias, cache: dict, out: torch.Tensor) -> None:
        plan, s, z = get_context().step, self.shape, offset["in"]
        hybrid_ops.state_space(s, proj, (z, z + s.inner, z + s.inner + s.channels), self.conv, self.conv_bias, self.dt_bias, self.a_log,
                               self.d, self.gain, cache["ring"], cache["state"], plan.state_slots, plan.positions, plan.decode_rows,
                               plan.spans, plan.max_span, plan.ring_slot, out)
