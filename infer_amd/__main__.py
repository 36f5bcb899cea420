"""Command line: greedy or sampled generation with a model of the registry.

    python -m infer_amd --model DIR --prompt "Hello"            (with a tokenizer in DIR)
    python -m infer_amd --model DIR --prompt-ids 5,17,3 --prompt-ids 8,1 --max-tokens 16
"""
from __future__ import annotations

import argparse
import json

from .llm_engine import LLMEngine
from .sampling_params import SamplingParams


def main(argv=None) -> None:
    ap = argparse.ArgumentParser(prog="python -m infer_amd", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--prompt", action="append", default=[], help="text prompt (repeatable)")
    ap.add_argument("--prompt-ids", action="append", default=[], help="comma-separated token ids (repeatable)")
    ap.add_argument("--max-tokens", type=int, default=64)
    ap.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    ap.add_argument("--ignore-eos", action="store_true")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], help="default: the model's")
    ap.add_argument("--block-size", type=int, default=256, help="tokens per cache block")
    ap.add_argument("--max-model-len", type=int, default=4096)
    ap.add_argument("--max-num-seqs", type=int, default=64)
    ap.add_argument("--max-batched-tokens", type=int, default=16384)
    ap.add_argument("--num-blocks", type=int, default=-1, help="cache blocks (default: what the memory holds)")
    ap.add_argument("--eager", action="store_true", help="no captured graphs")
    ap.add_argument("--seed", type=int, default=0)
    args = ap.parse_args(argv)
    prompts = args.prompt + [[int(t) for t in ids.split(",")] for ids in args.prompt_ids]
    if not prompts:
        ap.error("give at least one --prompt or --prompt-ids")
    engine = LLMEngine(args.model, dtype=args.dtype, kvcache_block_size=args.block_size, max_model_len=args.max_model_len,
                       max_num_seqs=args.max_num_seqs, max_num_batched_tokens=args.max_batched_tokens,
                       num_kvcache_blocks=args.num_blocks, enforce_eager=args.eager, seed=args.seed)
    params = SamplingParams(args.temperature, args.max_tokens, args.ignore_eos)
    for out in engine.generate(prompts, params):
        print(json.dumps(out))


if __name__ == "__main__":
    main()
