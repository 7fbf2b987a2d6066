#!/usr/bin/env python3
"""Prefill and decode throughput of the Dagupel design at the sizes of real models' layers (random weights), beside the
Llama step at equal width, heads and feed-forward; and each side's kernels against their rooflines.

    python bench.py --model dagupel [--sizes 2b,8b] [--layers 8] [--out FILE]

One JSON line per measurement.  Kernels are timed inside hipGraphs of one launch per layer (every layer has its own
weights and cache, so nothing is found in a cache); both models in turn in one process.
"""
from __future__ import annotations

import argparse
import dataclasses
import json
import os
import sys

import numpy as np
import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
from scalellm_amd import kernels, latent_kernels as lk  # noqa: E402
from scalellm_amd.dagupel import DagupelStep  # noqa: E402
from scalellm_amd.decode import LlamaDecodeStep, LlamaShape, make_batch_inputs, make_decode_inputs  # noqa: E402
from scalellm_amd.latent_layers import LatentPlan  # noqa: E402
from scalellm_amd.layers import Portion  # noqa: E402
from scalellm_amd.registry import ModelLimits  # noqa: E402

HBM, MFMA = 8.0e12, 2.5e15
DEV = "cuda"
BLOCK = 64

# name -> (width, heads, kv heads of the Llama beside it, ff, window)
SIZES = {"2b": (2048, 16, 8, 8192, 4096), "8b": (4096, 32, 8, 14336, 4096), "8b-w1k": (4096, 32, 8, 14336, 1024)}


class RandomCheckpoint:
    """Stands in for checkpoint.Checkpoint: random tensors of whatever shape is asked for."""

    def __init__(self, seed=0):
        self.g = torch.Generator(device=DEV).manual_seed(seed)

    def take(self, name, shape):
        if len(shape) == 1:
            return 1 + 0.1 * torch.randn(shape, device=DEV, generator=self.g)
        std = 1.0 if name in ("embed", "pos") else shape[1] ** -0.5
        return (torch.randn(shape, device=DEV, generator=self.g) * std).to(torch.bfloat16)

    def finish(self):
        pass


def dagupel(size, layers, n_blocks, max_positions=8192, vocab=32768):
    width, heads, _, ff, window = SIZES[size]
    layer = {"type": "latent_attention",
             "mixer": {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": 512, "mask": {"size": window},
                       "scale": 192 ** -0.5, "rot": {"base": 10000.0, "dims": 64,
                                                     "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}},
             "mlp": {"kind": "dense", "ff": ff, "limit": 7.0}}
    cfg = {"architecture": "Dagupel", "vocab": vocab, "width": width, "max_positions": max_positions, "norm": {"eps": 1e-5},
           "logit_scale": 1.0, "layers": [layer] * layers}
    m = DagupelStep.from_checkpoint(cfg, RandomCheckpoint(), ModelLimits(n_blocks, BLOCK, torch.bfloat16, DEV))
    for c in m.caches:
        c.rows.normal_()
    return m


def timed(fn, reps=5, graph=True):
    """Median seconds of fn(), replayed from a graph (or eager)."""
    fn()
    torch.cuda.synchronize()
    run = fn
    if graph:
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g):
            fn()
        run = g.replay
        run()
    ts = []
    for _ in range(reps):
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        run()
        b.record()
        b.synchronize()
        ts.append(a.elapsed_time(b) * 1e-3)
    return sorted(ts)[len(ts) // 2]


def batch(q_lens, kv_lens, block, vocab, portions):
    tokens, positions, params, n_blocks = make_batch_inputs(q_lens, kv_lens, block, DEV, seed=1, vocab=vocab)
    if portions:
        table, cu, row = params.block_tables.cpu().numpy(), params.cu_block_lens.cpu().numpy(), 0
        ps = []
        for i, (q, k) in enumerate(zip(q_lens, kv_lens)):
            ps.append(Portion(row, q, k, table[cu[i]:cu[i + 1]]))
            row += q
        params = dataclasses.replace(params, portions=ps)
    return tokens, positions, params, n_blocks


def llama(size, layers, n_blocks, max_tokens, vocab=32768):
    width, heads, kv_heads, ff, _ = SIZES[size]
    s = LlamaShape(hidden=width, n_heads=heads, n_kv_heads=kv_heads, head_dim=128, intermediate=ff, n_layers=layers, vocab=vocab,
                   max_position=8192)
    return LlamaDecodeStep(s, max_tokens, n_blocks, 16, dtype=torch.bfloat16, device=DEV, kv_fill="tile")


def visible_pairs(q_lens, kv_lens, window):
    n = 0
    for q, k in zip(q_lens, kv_lens):
        p = np.arange(k - q, k) + 1
        n += int((np.minimum(p, window) if window else p).sum())
    return n


def main(argv=None):
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", default="2b,8b")
    ap.add_argument("--layers", type=int, default=8)
    ap.add_argument("--decode", default="1,32,128", help="decode batch sizes")
    ap.add_argument("--context", type=int, default=4096)
    ap.add_argument("--prefill", default="1x4096,4x2048,8x512+3584", help="NxQ[+cached] prompt batches")
    ap.add_argument("--out", default="")
    ap.add_argument("--no-llama", action="store_true")
    args = ap.parse_args(argv)
    sink = open(args.out, "a") if args.out else None

    def emit(**rec):
        line = json.dumps({k: round(v, 4) if isinstance(v, float) else v for k, v in rec.items()})
        print(line, flush=True)
        if sink:
            sink.write(line + "\n")
            sink.flush()
    L = args.layers
    for size in args.sizes.split(","):
        width, heads, kv_heads, ff, window = SIZES[size]
        vocab = 32768
        cases = []
        for c in args.prefill.split(","):
            if c:
                n, q = c.split("x")
                q, cached = (q.split("+") + ["0"])[:2]
                cases.append((c, [int(q)] * int(n), [int(q) + int(cached)] * int(n)))
        sizes = [int(b) for b in args.decode.split(",") if b]
        need = max([b * (args.context + BLOCK) // BLOCK + 4 for b in sizes] + [sum(k) // BLOCK + len(k) + 4 for _, _, k in cases])
        for which in ("dagupel",) if args.no_llama else ("dagupel", "llama"):
            torch.cuda.empty_cache()
            D = which == "dagupel"
            block = BLOCK if D else 16
            most = max([sum(q) for _, q, _ in cases] + sizes)
            m = dagupel(size, L, need) if D else llama(size, L, need * (BLOCK // 16), most)
            base = dict(size=size, model=which, layers=L)
            # (the Llama step has no window: it decodes over as many keys as the window leaves the other)
            context = args.context if D else min(args.context, window)
            for bs in sizes:
                tokens, positions, params, _ = make_decode_inputs(bs, context, block, DEV, seed=1, vocab=vocab)
                if D:
                    m.reserve_workspaces(bs)
                else:
                    m.reserve_workspaces(bs, context)
                t = timed(lambda: m.forward(tokens, positions, params))
                emit(kind="decode", **base, bs=bs, context=context, ms=t * 1e3, us_per_layer=t / L * 1e6, tokens_per_s=bs / t)
                # the kernels of a layer
                if D:
                    a0 = m.layers[0].attn
                    R = a0.c_pad + a0.r_pad
                    q = torch.randn(bs, heads, R, device=DEV).to(torch.bfloat16)
                    o = torch.empty(bs, heads, a0.c_pad, dtype=torch.bfloat16, device=DEV)

                    def attn():
                        for c in m.caches:
                            lk.latent_attention(q, c.rows, o, positions, params.q_cu_seq_lens, params.block_tables, params.cu_block_lens,
                                                block_size=BLOCK, window=window, scale=0.07, max_kv_len=context)
                    seen = min(window, context)
                    nbytes, flops = bs * seen * R * 2, 2 * bs * seen * heads * (R + a0.c_pad)
                    h = torch.randn(bs, m.k_width, device=DEV).to(torch.bfloat16)
                    act = torch.randn(bs, ff, device=DEV).to(torch.bfloat16)
                    lins = {"proj": lambda: [lk.linear(h, x.attn.w_in) for x in m.layers],
                            "gate_up+act": lambda: [lk.linear_glu(h, x.mlp.w_gate_up, act, 7.0) for x in m.layers],
                            "down": lambda: [x.mlp.w_down is not None and (lk.linear_slabs if bs <= lk.STREAM_MAX_ROWS else lk.linear)(act, x.mlp.w_down)
                                             for x in m.layers]}
                    wbytes = {"proj": a0.w_in.numel() * 2, "gate_up+act": m.layers[0].mlp.w_gate_up.numel() * 2,
                              "down": m.layers[0].mlp.w_down.numel() * 2}
                    wflops = {k: bs * v for k, v in wbytes.items()}
                else:
                    q = torch.randn(bs, heads, 128, device=DEV).to(torch.bfloat16)
                    o = torch.empty_like(q)

                    def attn():
                        for x in m.layers:
                            m.attn.handler.batch_decode(q, x["kv"], params, -1, o)
                    seen = context
                    nbytes, flops = bs * seen * kv_heads * 128 * 4, 4 * bs * seen * heads * 128
                    h = torch.randn(bs, width, device=DEV).to(torch.bfloat16)
                    act = torch.randn(bs, ff, device=DEV).to(torch.bfloat16)
                    lins = {"proj": lambda: [x["qkv"].forward(h, out=m.buf["qkv"][:bs]) for x in m.layers],
                            "gate_up+act": lambda: [x["gate_up"].forward(h, out=m.buf["act"][:bs]) for x in m.layers],
                            "down": lambda: [x["down"].forward(act, out=m.buf["down"][:bs], reduce=False, defer_splitk=True) for x in m.layers]}
                    pk = {"proj": "qkv", "gate_up+act": "gate_up", "down": "down"}
                    wbytes = {k: m.layers[0][v]._packed.wq.numel() * m.layers[0][v]._packed.wq.element_size() +
                              m.layers[0][v]._packed.sz.numel() * m.layers[0][v]._packed.sz.element_size() for k, v in pk.items()}
                    wflops = {k: 2 * bs * (heads + 2 * kv_heads) * 128 * width if k == "proj" else
                              2 * bs * width * ff * (2 if k != "down" else 1) for k in wbytes}
                t = timed(attn) / L
                roof = max(nbytes / HBM, flops / MFMA)
                emit(kind="kernel", **base, kernel="decode attention", bs=bs, us=t * 1e6, tb_per_s=nbytes / t / 1e12,
                     tflops=flops / t / 1e12, roofline=roof / t)
                for name, fn in lins.items():
                    t = timed(fn) / L
                    roof = max(wbytes[name] / HBM, wflops[name] / MFMA)
                    emit(kind="kernel", **base, kernel=name, bs=bs, us=t * 1e6, tb_per_s=wbytes[name] / t / 1e12,
                         tflops=wflops[name] / t / 1e12, roofline=roof / t)
            for name, q_lens, kv_lens in cases:
                tokens, positions, params, _ = batch(q_lens, kv_lens, block, vocab, D)
                T = tokens.numel()
                if not D:
                    m.reserve_workspaces(T, max(kv_lens))
                t = timed(lambda: m.forward(tokens, positions, params), graph=False)
                emit(kind="prefill", **base, batch=name, tokens=T, ms=t * 1e3, us_per_layer=t / L * 1e6, tokens_per_s=T / t)
                if D:
                    a0 = m.layers[0].attn
                    proj = torch.randn(T, a0.w_in.size(0), device=DEV).to(torch.bfloat16)
                    out = torch.empty(T, a0.o_k, dtype=torch.bfloat16, device=DEV)
                    plan = LatentPlan.build(params.portions, window, BLOCK, DEV)
                    ctx = lk.latent_gather(m.caches[0].rows, plan.slots)
                    kv = torch.mm(ctx[:, :a0.c_pad], a0.w_ukv.t())

                    def attn():
                        for _ in range(L):
                            lk.latent_prefill(proj, ctx, kv, out, plan.tiles, heads=heads, q_dim=a0.q_dim, c_pad=a0.c_pad,
                                              v_pad=a0.v_pad, gate_off=a0.off_g, window=window, scale=0.07)
                    flops = 2 * visible_pairs(q_lens, kv_lens, window) * heads * (a0.head_w + a0.v_pad)
                    t = timed(lambda: [lk.latent_gather(c.rows, plan.slots) for c in m.caches]) / L
                    nb = 2 * ctx.numel() * 2
                    emit(kind="kernel", **base, kernel="gather context", batch=name, us=t * 1e6, tb_per_s=nb / t / 1e12, roofline=nb / HBM / t)
                    t = timed(lambda: [torch.mm(ctx[:, :a0.c_pad], x.attn.w_ukv.t()) for x in m.layers]) / L
                    fl = 2 * ctx.size(0) * a0.w_ukv.numel()
                    emit(kind="kernel", **base, kernel="expand context (vendor)", batch=name, us=t * 1e6, tflops=fl / t / 1e12, roofline=fl / MFMA / t)
                else:
                    q = torch.randn(T, heads, 128, device=DEV).to(torch.bfloat16)
                    o = torch.empty_like(q)

                    def attn():
                        for x in m.layers:
                            m.attn.handler.batch_decode(q, x["kv"], params, -1, o)
                    flops = 4 * visible_pairs(q_lens, kv_lens, 0) * heads * 128
                t = timed(attn) / L
                emit(kind="kernel", **base, kernel="prompt attention", batch=name, us=t * 1e6, tflops=flops / t / 1e12,
                     roofline=flops / MFMA / t)
                if D:
                    h = torch.randn(T, m.k_width, device=DEV).to(torch.bfloat16)
                    act = torch.empty(T, ff, device=DEV, dtype=torch.bfloat16)
                    t = timed(lambda: [lk.linear_glu(h, x.mlp.w_gate_up, act, 7.0) for x in m.layers]) / L
                else:
                    h = torch.randn(T, width, device=DEV).to(torch.bfloat16)
                    t = timed(lambda: [x["gate_up"].forward(h, out=m.buf["act"][:T]) for x in m.layers]) / L
                fl = 4 * T * width * ff
                emit(kind="kernel", **base, kernel="gate_up+act", batch=name, us=t * 1e6, tflops=fl / t / 1e12, roofline=fl / MFMA / t)
            del m
    return 0


if __name__ == "__main__":
    sys.exit(main())
