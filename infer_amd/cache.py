"""What a model keeps between steps, and how much memory it takes.

A model says what every layer needs (``cache_layout``); the runner sizes the pool from the sum, allocates it and
hands every layer its part.  Two kinds of storage exist: pages, which belong to cache blocks and grow with a
sequence, and slots, which hold a fixed amount per running sequence."""
from __future__ import annotations

import math

import torch

from . import kv_runner


class PagedKVLayout:
    """K and V pages of equal layers, in one tensor ``[2, layers, blocks, block_size, heads, head_dim]``."""
    slot_bytes = 0

    def __init__(self, num_layers: int, block_size: int, num_kv_heads: int, head_dim: int, dtype: torch.dtype):
        self.args = (num_layers, block_size, num_kv_heads, head_dim)
        self.dtype = dtype
        self.block_bytes = kv_runner.kv_block_bytes(*self.args, dtype.itemsize)

    def allocate(self, num_blocks: int, num_slots: int, device) -> torch.Tensor:
        return kv_runner.allocate_kv_cache(num_blocks, *self.args, device, self.dtype)


class LatentPages:
    """One row of ``row`` elements per token, shared by all heads of a layer."""

    def __init__(self, row: int, dtype: torch.dtype):
        self.row, self.dtype = row, dtype

    def block_bytes(self, block_size: int) -> int:
        return block_size * self.row * self.dtype.itemsize

    slot_bytes = 0

    def allocate(self, num_blocks: int, num_slots: int, block_size: int, device):
        return torch.zeros(num_blocks, block_size, self.row, dtype=self.dtype, device=device)


class GroupedPages:
    """A row ``[value | key]`` of ``row`` elements per token and key/value head."""

    def __init__(self, kv_heads: int, row: int, dtype: torch.dtype):
        self.kv_heads, self.row, self.dtype = kv_heads, row, dtype

    def block_bytes(self, block_size: int) -> int:
        return block_size * self.kv_heads * self.row * self.dtype.itemsize

    slot_bytes = 0

    def allocate(self, num_blocks: int, num_slots: int, block_size: int, device):
        return torch.zeros(num_blocks, self.kv_heads, block_size, self.row, dtype=self.dtype, device=device)


class TilePages:
    """Keys and values per token and key/value head in pages of their own, in tiles of 32 tokens that matrix operands read as they lie:
    keys of ``key_row`` entries as ``[tile][key_row / 8][token][8]``, values as ``[tile][value_row / 16][token / 8][16][8 tokens]``."""
    TOKENS = 32
    slot_bytes = 0

    def __init__(self, kv_heads: int, key_row: int, value_row: int, dtype: torch.dtype):
        assert key_row % 32 == value_row % 32 == 0
        self.kv_heads, self.key_row, self.value_row, self.dtype = kv_heads, key_row, value_row, dtype

    def block_bytes(self, block_size: int) -> int:
        return block_size * self.kv_heads * (self.key_row + self.value_row) * self.dtype.itemsize

    def allocate(self, num_blocks: int, num_slots: int, block_size: int, device):
        tiles = (num_blocks, self.kv_heads, block_size // self.TOKENS)
        return {"keys": torch.zeros(*tiles, self.key_row // 8, self.TOKENS, 8, dtype=self.dtype, device=device),
                "values": torch.zeros(*tiles, self.value_row // 16, 4, 16, 8, dtype=self.dtype, device=device)}


class SharedStorage:
    """A layer that keeps nothing of its own and reads what the earlier layer ``owner`` keeps."""
    slot_bytes = 0

    def __init__(self, owner: int):
        self.owner = owner

    def block_bytes(self, block_size: int) -> int:
        return 0


class StateSlots:
    """Named tensors per running sequence: ``name=(shape, dtype)``."""

    def __init__(self, **tensors):
        self.tensors = tensors

    def block_bytes(self, block_size: int) -> int:
        return 0

    @property
    def slot_bytes(self) -> int:
        return sum(math.prod(shape) * dtype.itemsize for shape, dtype in self.tensors.values())

    def allocate(self, num_blocks: int, num_slots: int, block_size: int, device):
        return {name: torch.zeros(num_slots, *shape, dtype=dtype, device=device)
                for name, (shape, dtype) in self.tensors.items()}


class StorageGroup:
    """What several parts of one layer keep, by name."""

    def __init__(self, parts: dict):
        self.parts = parts
        self.slot_bytes = sum(p.slot_bytes for p in parts.values())

    def block_bytes(self, block_size: int) -> int:
        return sum(p.block_bytes(block_size) for p in self.parts.values())

    def allocate(self, num_blocks: int, num_slots: int, block_size: int, device):
        return {name: p.allocate(num_blocks, num_slots, block_size, device) for name, p in self.parts.items()}


class LayeredLayout:
    """One storage description per layer; ``allocate`` returns one storage per layer."""

    def __init__(self, layers: list, block_size: int):
        self.layers, self.block_size = layers, block_size
        self.block_bytes = sum(layer.block_bytes(block_size) for layer in layers)
        self.slot_bytes = sum(layer.slot_bytes for layer in layers)

    def allocate(self, num_blocks: int, num_slots: int, device) -> list:
        storage: list = []
        for layer in self.layers:
            shared = isinstance(layer, SharedStorage)
            storage.append(storage[layer.owner] if shared else layer.allocate(num_blocks, num_slots, self.block_size, device))
        return storage
