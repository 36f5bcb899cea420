"""Device metadata of one step of a model that runs portions of prompts beside decoded tokens.

The rows of the batch are the portions' tokens, portions sorted by length (decoded tokens, one row each,
come first).  All arrays of a step travel in one pinned buffer and one copy."""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

# Portions of at least this many tokens attend over keys and values expanded from the latents of their whole
# sequence; the tokens of shorter ones attend over the latents themselves, one by one, as decoded tokens do.
DENSE_FROM = 64
CHUNK = 16          # tokens per chunk of a recurrent layer's prompt kernels


@dataclass
class StepPlan:
    input_ids: torch.Tensor                # int64 [rows]
    positions: torch.Tensor                # int64 [rows]
    slot_mapping: torch.Tensor             # int32 [rows] cache row of each token, -1: padding
    block_tables: torch.Tensor             # int32 [sequences, columns]
    row_ctx: torch.Tensor                  # int32 [rows] keys each row sees
    state_slots: torch.Tensor              # int32 [decode_rows]
    prev_ids: torch.Tensor                 # int64 [rows] the token in front of each in its sequence, -1: none
    decode_rows: int                       # rows that are the only one of their portion
    row_seq: torch.Tensor | None = None    # int32 [rows] block-table row of each row; None: the row itself
    max_keys: int | None = None            # largest row_ctx, where the host knows it
    # recurrent layers: the rows behind decode_rows (descriptors of ``hybrid_ops.delta_chunks``)
    portions: torch.Tensor | None = None
    chunks: torch.Tensor | None = None
    ring_slot: torch.Tensor | None = None
    spans: torch.Tensor | None = None      # int32 [.., 4] first row, tokens, state slot, first position (``hybrid_ops.decay_attention``)
    max_span: int = 0                      # tokens of the longest
    # attention: rows from dense_row on belong to long portions
    dense_row: int = 0
    dense_seqs: torch.Tensor | None = None      # int32, block-table rows
    dense_cu_q: torch.Tensor | None = None      # int32, relative to dense_row
    dense_cu_k: torch.Tensor | None = None
    dense_keys: int = 0
    dense_max_q: int = 0
    dense_max_k: int = 0

    @property
    def rows(self) -> int:
        return self.positions.numel()


def build(portions, block_size: int, max_blocks: int, num_slots: int, num_blocks: int, device):
    """``portions``: (sequence, count) pairs.  Returns the plan and, for every portion in the given order, the first
    batch row of its tokens."""
    order = sorted(range(len(portions)), key=lambda i: portions[i][1])
    counts = [portions[i][1] for i in order]
    first = np.concatenate(([0], np.cumsum(counts)))
    rows = int(first[-1])
    ids, pos, prev = (np.empty(rows, np.int64) for _ in range(3))
    slots, row_seq = np.empty(rows, np.int32), np.empty(rows, np.int32)
    ring = np.empty((rows, 2), np.int32)
    tables = np.zeros((len(order), max(1, max(len(portions[i][0].block_table) for i in order))), np.int32)
    port, chunk, span, dense = [], [], [], []
    for s, i in enumerate(order):
        seq, n = portions[i]
        lo, r0 = seq.num_computed_tokens, int(first[s])
        table = np.asarray(seq.block_table, np.int32)
        if n < 1 or lo + n > len(table) * block_size or len(table) > max_blocks:
            raise RuntimeError(f"portion of {n} tokens at {lo} does not fit {len(table)} cache blocks")
        if table.min() < 0 or table.max() >= num_blocks or not 0 <= seq.state_slot < num_slots:
            raise RuntimeError("a portion's cache blocks or state slot lie outside the pool")
        tables[s, :len(table)] = table
        p = np.arange(lo, lo + n)
        ids[r0:r0 + n] = seq.token_ids[lo:lo + n]
        pos[r0:r0 + n] = p
        prev[r0] = seq.token_ids[lo - 1] if lo else -1
        prev[r0 + 1:r0 + n] = ids[r0:r0 + n - 1]
        slots[r0:r0 + n] = table[p // block_size] * block_size + p % block_size
        row_seq[r0:r0 + n] = s
        ring[r0:r0 + n, 0] = seq.state_slot
        ring[r0:r0 + n, 1] = np.arange(n - 1, -1, -1)       # rows of the portion that follow
        if n > 1:
            port.append((len(chunk), -(-n // CHUNK), seq.state_slot, lo))
            span.append((r0, n, seq.state_slot, lo))
            chunk += [(r0 + c, min(CHUNK, n - c), lo + c, lo, seq.state_slot, 0) for c in range(0, n, CHUNK)]
        if n >= DENSE_FROM:
            dense.append(s)
    decode_rows = sum(1 for n in counts if n == 1)
    dense_row = int(first[dense[0]]) if dense else rows
    parts = {"ids": ids, "pos": pos, "prev": prev, "slots": slots, "tables": tables, "row_seq": row_seq,
             "ctx": (pos + 1).astype(np.int32), "ring": ring,
             "state": ring[:decode_rows, 0],
             "port": np.asarray(port, np.int32).reshape(-1, 4), "chunk": np.asarray(chunk, np.int32).reshape(-1, 6),
             "span": np.asarray(span, np.int32).reshape(-1, 4), "dense": np.asarray(dense, np.int32)}
    ends = [portions[order[s]][0].num_computed_tokens + counts[s] for s in dense]
    parts["cu_q"] = np.concatenate(([0], np.cumsum([counts[s] for s in dense]))).astype(np.int32)
    parts["cu_k"] = np.concatenate(([0], np.cumsum(ends))).astype(np.int32)
    t = _upload(parts, device)
    plan = StepPlan(input_ids=t["ids"], positions=t["pos"], slot_mapping=t["slots"], block_tables=t["tables"],
                    row_ctx=t["ctx"], state_slots=t["state"], prev_ids=t["prev"], decode_rows=decode_rows, row_seq=t["row_seq"],
                    max_keys=int(pos.max()) + 1, portions=t["port"], chunks=t["chunk"], ring_slot=t["ring"],
                    spans=t["span"], max_span=max((n for _, n, _, _ in span), default=0),
                    dense_row=dense_row, dense_seqs=t["dense"], dense_cu_q=t["cu_q"], dense_cu_k=t["cu_k"],
                    dense_keys=int(sum(ends)), dense_max_q=max((counts[s] for s in dense), default=0),
                    dense_max_k=max(ends, default=0))
    start = [0] * len(portions)
    for s, i in enumerate(order):
        start[i] = int(first[s])
    return plan, start


def _upload(parts: dict, device) -> dict:
    """All arrays in one pinned buffer and one copy; every array starts on 16 bytes."""
    device = torch.device(device)
    offsets, total = {}, 0
    for name, a in parts.items():
        offsets[name] = total
        total += -(-a.nbytes // 16) * 16
    host = torch.empty(max(total, 16), dtype=torch.uint8, pin_memory=device.type == "cuda")
    raw = host.numpy()
    for name, a in parts.items():
        raw[offsets[name]:offsets[name] + a.nbytes] = np.ascontiguousarray(a).reshape(-1).view(np.uint8)
    dev = host.to(device, non_blocking=True)
    out = {}
    for name, a in parts.items():
        dtype = torch.int64 if a.dtype == np.int64 else torch.int32
        out[name] = dev[offsets[name]:offsets[name] + a.nbytes].view(dtype).view(a.shape)
    return out
