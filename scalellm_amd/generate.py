"""Command line: generate token ids from a model folder.

    python -m scalellm_amd.generate --model DIR --prompt 5,17,3 [--prompt ...] [--max-tokens 32] [--temperature 0.8 ...]

Prompts are token ids (the folder holds no tokenizer); one JSON line per prompt: {"prompt": [...], "tokens": [...]}.
"""
from __future__ import annotations

import argparse
import json
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="scalellm_amd.generate", description="generate token ids from a model folder")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--prompt", action="append", required=True, help="comma-separated token ids (repeatable)")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--max-tokens", type=int, default=32, help="tokens to generate per prompt")
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--top-k", type=int, default=0)
    ap.add_argument("--top-p", type=float, default=1.0)
    ap.add_argument("--seed", type=int, default=None)
    ap.add_argument("--stop", type=int, action="append", default=[], help="token id that ends a sequence (repeatable)")
    ap.add_argument("--block-size", type=int, default=64)
    ap.add_argument("--cache-tokens", type=int, default=0, help="size of the cache pool (default: what the prompts need)")
    ap.add_argument("--max-seqs", type=int, default=64, help="sequences served together")
    ap.add_argument("--step-tokens", type=int, default=2048, help="token budget of a step")
    ap.add_argument("--graphs", default="", help="decode batch sizes to capture into hipGraphs, comma-separated")
    args = ap.parse_args(argv)
    prompts = [[int(t) for t in p.split(",") if t.strip()] for p in args.prompt]

    import torch
    from .engine import EngineOptions, LLMEngine
    from .registry import ModelLimits, load_model
    from .sampling import SamplingParams
    B = args.block_size
    longest = max(len(p) for p in prompts) + args.max_tokens
    blocks = args.cache_tokens // B if args.cache_tokens else sum((len(p) + args.max_tokens + B - 1) // B for p in prompts)
    graphs = [int(g) for g in args.graphs.split(",") if g]
    model = load_model(args.model, ModelLimits(max(blocks, 1), B, getattr(torch, args.dtype), "cuda", n_states=args.max_seqs,
                                                max_positions=longest))
    engine = LLMEngine(model, max(blocks, 1), B, "cuda", EngineOptions(
        max_seqs=args.max_seqs, max_step_tokens=args.step_tokens, graph_batch_sizes=graphs, graph_max_seq_len=longest))
    engine.capture_graphs()
    out = engine.generate(prompts, SamplingParams(args.max_tokens, args.temperature, args.top_k, args.top_p, args.seed, args.stop))
    for p, t in zip(prompts, out):
        print(json.dumps({"prompt": p, "tokens": t}), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
