"""Replays recorded steps through the engine: given tokens in, logits out, nothing sampled.

A step names, per request, its next tokens and the places among them whose logits are wanted.  Placement, cache
blocks, state slots and the forward pass are the engine's own (``PortionScheduler.place``,
``ModelRunner.portion_logits``); only the choice of what runs in a step comes from the trace."""
from __future__ import annotations

import json
import os

import torch

from .llm_engine import LLMEngine
from .scheduler import Portion
from .sequence import Sequence

BLOCK = 64


class TraceReplay:

    def __init__(self, model: str, dtype: str, max_tokens: int, max_requests: int = 4):
        blocks = -(-max_tokens // BLOCK)
        self.engine = LLMEngine(model, dtype=dtype, kvcache_block_size=BLOCK, num_kvcache_blocks=blocks,
                                max_num_seqs=max_requests, max_model_len=blocks * BLOCK, max_num_batched_tokens=blocks * BLOCK)
        if not self.engine.model_runner.mixed:
            raise RuntimeError("traces of portions need a model that runs portions")
        self.live: dict[str, Sequence] = {}

    def step(self, entries: list[dict], end: list[str]) -> torch.Tensor | None:
        """Runs one step.  Returns the wanted logits as float32 on the host, None if nothing is wanted."""
        scheduler = self.engine.scheduler
        portions, wanted = [], []
        for entry in entries:
            tokens, seq = entry["tokens"], self.live.get(entry["id"])
            if not tokens:
                continue
            if seq is None:
                seq = self.live[entry["id"]] = Sequence(tokens, block_size=BLOCK)
                scheduler.start(seq)
            else:
                for token in tokens:
                    seq.append_token(token)
            if not scheduler.place(seq, len(tokens)):
                raise RuntimeError(f"no room for {len(tokens)} tokens of request {entry['id']}")
            portions.append(Portion(seq, len(tokens)))
            wanted.append(entry.get("want", []))
        logits = None
        if portions:
            rows = self.engine.model_runner.portion_logits(portions, wanted)
            scheduler.advance(portions)
            if any(wanted):
                logits = rows.float().cpu()
        for name in end:
            seq = self.live.pop(name, None)
            if seq is not None:
                scheduler.finish(seq)
        return logits


def replay(model: str, dtype: str, out: str, max_tokens: int, lines) -> None:
    """Reads steps (one JSON object a line), writes ``<step>.f32`` for every step that wants logits and prints
    ``done <step>`` after each."""
    trace = TraceReplay(model, dtype, max_tokens)
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        logits = trace.step(step["entries"], step.get("end", []))
        if logits is not None:
            logits.contiguous().numpy().astype("<f4").tofile(os.path.join(out, f"{step['step']}.f32"))
        print("done", step["step"], flush=True)
