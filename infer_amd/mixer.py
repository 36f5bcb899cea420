"""A layer's mixer made of one or more parts that read the same input and whose results are added.

All parts share one input product and one output product.  A part names the projections it wants (``pieces``) and what it keeps
between steps (``cache_spec``), and turns its columns of the input product into its columns of the output product's input."""
from __future__ import annotations

import torch
from torch import nn

from .cache import StorageGroup
from .layers import ColumnPackedLinear, PackedBias, PackedLinear

MAIN = "main"          # the name of a part that is alone


class Mixer(nn.Module):

    def __init__(self, hidden_size: int, parts: dict, dtype: torch.dtype):
        super().__init__()
        self.parts = nn.ModuleDict(parts)
        pieces = {self.piece(name, key): size for name, part in parts.items() for key, size in part.pieces().items()}
        dense = tuple(self.piece(name, key) for name, part in parts.items() for key in part.dense_pieces)
        self.in_proj = PackedLinear(hidden_size, pieces, dtype, dense=dense)
        self.o_proj = ColumnPackedLinear({name: part.out_size for name, part in parts.items()}, hidden_size, dtype)
        biased = tuple(self.piece(name, key) for name, part in parts.items() for key in part.biased_pieces)
        self.bias = PackedBias(self.in_proj, biased) if biased else None

    @staticmethod
    def piece(part: str, key: str) -> str:
        return key if part == MAIN else f"{part}.{key}"

    def cache_spec(self):
        return StorageGroup({name: part.cache_spec() for name, part in self.parts.items()})

    def finish_loading(self, max_position: int) -> None:
        for part in self.parts.values():
            part.finish_loading(max_position)

    def forward(self, h: torch.Tensor, storage: dict) -> torch.Tensor:
        proj = self.in_proj(h)
        out = (torch.zeros if self.o_proj.padded else torch.empty)((h.shape[0], self.o_proj.in_features), dtype=h.dtype, device=h.device)
        bias = self.bias.weight if self.bias is not None else None
        for name, part in self.parts.items():
            offset = {key: self.in_proj.offset[self.piece(name, key)] for key in part.pieces()}
            part(proj, offset, bias, storage[name], out[:, self.o_proj.offset[name]:])
        return self.o_proj(out, defer=True)
