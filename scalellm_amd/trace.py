"""Replay of a request trace: given token ids through a model, step by step, logits to files.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come as JSON lines on standard input:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
All entries of a step are one batch of LLMEngine.run_entries.  Wanted logits go to OUT/<step>.f32 (little-endian
fp32 [wanted, vocab], entries and places in the given order); "done <step>" is printed after every step.  Requests
named in "end" give their cache blocks and state back.  --max-tokens sizes the pool: the most tokens live requests hold, each
rounded up to the block size.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

BLOCK_SIZE = 64
MAX_REQUESTS = 4


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a request trace and write its logits")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True)
    ap.add_argument("--max-tokens", required=True, type=int, help="size of the cache pool in tokens")
    args = ap.parse_args(argv)

    import torch
    from .engine import EngineOptions, LLMEngine, Sequence
    from .registry import ModelLimits, load_model
    if not torch.cuda.is_available():
        print("trace_run needs a GPU", file=sys.stderr)
        return 2
    n_blocks = max(1, (args.max_tokens + BLOCK_SIZE - 1) // BLOCK_SIZE)
    limits = ModelLimits(n_blocks, BLOCK_SIZE, getattr(torch, args.dtype), "cuda", n_states=MAX_REQUESTS)
    engine = LLMEngine(load_model(args.model, limits), n_blocks, BLOCK_SIZE, "cuda", EngineOptions(max_seqs=MAX_REQUESTS))
    live = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        req = json.loads(line)
        entries, wanted = [], {}
        for k, e in enumerate(req["entries"]):
            seq = live.get(e["id"])
            if seq is None:
                if len(live) >= MAX_REQUESTS:
                    raise RuntimeError(f"more than {MAX_REQUESTS} live requests")
                seq = live[e["id"]] = Sequence(e["id"], [])
            engine.check_tokens(e["tokens"], len(seq.tokens))
            seq.tokens += e["tokens"]
            entries.append((seq, len(e["tokens"])))
            wanted[k] = e["want"]
        if entries:
            _, logits = engine.run_entries(entries, wanted)
            if any(wanted.values()):
                data = logits.float().cpu().contiguous().numpy().astype("<f4")
                with open(os.path.join(args.out, f"{req['step']}.f32"), "wb") as f:
                    f.write(data.tobytes())
            else:
                torch.cuda.synchronize()
        for name in req.get("end", []):
            live.pop(name).release(engine.allocator)
        print(f"done {req['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
