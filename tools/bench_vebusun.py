#!/usr/bin/env python3
"""Prefill and decode throughput of the Vebusun design at the sizes of real models' layers (random weights), beside the
Dagupel step (its neighbour on the dense 16-bit path) and the Llama step at equal width, heads and feed-forward; and each
kernel against its roofline.

    python bench.py --model vebusun [--sizes 2b,8b] [--layers 8] [--out FILE]

A quarter of the Vebusun layers are parallel ones (three delta layers, then one).  One JSON line per measurement.  Kernels
are timed inside hipGraphs of one launch per layer (every layer has its own weights, cache and state).
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
from scalellm_amd import latent_kernels as lk, mixer_kernels as mk  # noqa: E402
from scalellm_amd.decode import make_decode_inputs  # noqa: E402
from scalellm_amd.mixer_layers import ChannelDelta, WindowPlan  # noqa: E402
from scalellm_amd.registry import ModelLimits  # noqa: E402
from scalellm_amd.vebusun import VebusunStep  # noqa: E402
from tools.bench_dagupel import BLOCK, DEV, HBM, MFMA, SIZES, RandomCheckpoint, batch, dagupel, llama, timed, visible_pairs  # noqa: E402

FP32 = 157.3e12   # 32-bit matrix products
KEEP = 16


class Weights(RandomCheckpoint):
    def names(self):
        return ()

    def take(self, name, shape=None):
        if name.endswith(".alpha"):
            return torch.tensor(0.5)
        if shape is None:   # (the low-rank pairs: the rank is the tensors' own)
            shape = (128, self.width)
        if name.endswith("dt_bias"):
            return torch.full(shape, -4.0, device=DEV)
        return super().take(name, shape)


def vebusun(size, layers, n_blocks, n_states, vocab=32768):
    width, heads, kv_heads, ff, window = SIZES[size]
    mlp = {"kind": "dense", "ff": ff}
    delta = {"type": "channel_delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": heads, "dim": 128, "vdim": 128, "conv": 4}}
    both = {"type": "parallel", "mlp": mlp, "mixer": {
        "left_scale": 0.7, "right_scale": 0.7,
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 30.0,
                 "rot": {"base": 10000.0, "dims": 128}, "mask": {"size": window, "keep_first": KEEP}},
        "right": {"heads": heads, "dim": 128, "vdim": 128, "decay": [1 - 2.0 ** -(5 + 4 * h / heads) for h in range(heads)]}}}
    cfg = {"architecture": "Vebusun", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": 1.0},
           "residual_mult": 0.3, "loop": None, "layers": [both if i % 4 == 3 else delta for i in range(layers)]}
    w = Weights()
    w.width = width
    m = VebusunStep.from_checkpoint(cfg, w, ModelLimits(n_blocks, BLOCK, torch.bfloat16, DEV, n_states, max_positions=16384))
    for c in m.caches:
        if isinstance(c, tuple):
            for t in c[0].get_kv_cache():
                t.normal_()
    return m


def with_states(params):
    import dataclasses
    return dataclasses.replace(params, state_slots=torch.arange(params.q_cu_seq_lens.numel() - 1, dtype=torch.int32, device=DEV))


def main(argv=None):
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", default="2b,8b")
    ap.add_argument("--layers", type=int, default=8)
    ap.add_argument("--decode", default="1,32,128", help="decode batch sizes")
    ap.add_argument("--context", type=int, default=4096)
    ap.add_argument("--prefill", default="1x4096,4x2048,8x512+3584", help="NxQ[+cached] prompt batches")
    ap.add_argument("--out", default="")
    ap.add_argument("--models", default="vebusun,dagupel,llama")
    args = ap.parse_args(argv)
    sink = open(args.out, "a") if args.out else None

    def emit(**rec):
        line = json.dumps({k: round(v, 4) if isinstance(v, float) else v for k, v in rec.items()})
        print(line, flush=True)
        if sink:
            sink.write(line + "\n")
            sink.flush()
    L, vocab = args.layers, 32768
    for size in args.sizes.split(","):
        width, heads, kv_heads, ff, window = SIZES[size]
        cases = []
        for c in args.prefill.split(","):
            if c:
                n, q = c.split("x")
                q, cached = (q.split("+") + ["0"])[:2]
                cases.append((c, [int(q)] * int(n), [int(q) + int(cached)] * int(n)))
        sizes = [int(b) for b in args.decode.split(",") if b]
        need = max([b * (args.context + BLOCK) // BLOCK + 4 for b in sizes] + [sum(k) // BLOCK + len(k) + 4 for _, _, k in cases])
        most = max([sum(q) for _, q, _ in cases] + sizes)
        for which in args.models.split(","):
            torch.cuda.empty_cache()
            V = which == "vebusun"
            block = 16 if which == "llama" else BLOCK
            m = (vebusun(size, L, need, max(sizes + [8])) if V else dagupel(size, L, need) if which == "dagupel" else
                 llama(size, L, need * (BLOCK // 16), most))
            base = dict(size=size, model=which, layers=L)

            def kernel(name, fn, count, nbytes=0, flops=0, fp32=0, **rec):
                t = timed(fn) / count
                roof = max(nbytes / HBM, flops / MFMA, fp32 / FP32)
                emit(kind="kernel", **base, kernel=name, us=t * 1e6, tb_per_s=nbytes / t / 1e12, tflops=(flops + fp32) / t / 1e12,
                     roofline=roof / t, **rec)
            if V:
                pairs = list(zip(m.layers, m.caches))
                deltas = [(x, c) for x, c in pairs if isinstance(x.mixer, ChannelDelta)]
                paras = [(x, c) for x, c in pairs if not isinstance(x.mixer, ChannelDelta)]
                d0, p0 = deltas[0][0].mixer, paras[0][0].mixer
                S = heads * 128 * 128
                chunk_flops = 3 * 2 * S + 2 * heads * (2 * 16 * 128 + 2 * 16 * 128)
            for bs in sizes:
                context = args.context if which != "llama" else min(args.context, window)
                tokens, positions, params, _ = make_decode_inputs(bs, context, block, DEV, seed=1, vocab=vocab)
                if V:
                    params = with_states(params)
                m.reserve_workspaces(bs) if which != "llama" else m.reserve_workspaces(bs, context)
                t = timed(lambda: m.forward(tokens, positions, params))
                emit(kind="decode", **base, bs=bs, context=context, ms=t * 1e3, us_per_layer=t / L * 1e6, tokens_per_s=bs / t)
                if not V:
                    continue
                h = torch.randn(bs, m.k_width, device=DEV).to(torch.bfloat16)
                projd, projp = lk.linear(h, d0.w_in), lk.linear(h, p0.w_in)
                low = torch.randn(bs, 2 * d0.low_n, device=DEV).to(torch.bfloat16)
                out = torch.empty(bs, d0.o_k, device=DEV, dtype=torch.bfloat16)
                step = (positions, params.q_cu_seq_lens, params.state_slots, bs)
                kernel("delta step", lambda: [mk.recurrent_step(x.mixer.spec, projd, low, c, *step, out=out) for x, c in deltas], len(deltas),
                       nbytes=bs * (8 * S + 2 * 4 * 3 * heads * 128 + 2 * 8 * heads * 128), bs=bs)
                right = projp[:, p0.split:]
                kernel("lightning step", lambda: [mk.recurrent_step(x.mixer.right.spec, right, None, c[1], *step) for x, c in paras], len(paras),
                       nbytes=bs * (8 * S + 2 * 3 * heads * 128), bs=bs)
                o = torch.randn(bs, heads, 128, device=DEV)
                kernel("norm + gate", lambda: [mk.gated_norm(o, 128, right[:, p0.right.off_g:], x.mixer.right.norm, out, eps=1e-5, per_head=False)
                                               for x, c in paras], len(paras), nbytes=bs * heads * 128 * 8, bs=bs)
                a = p0.left
                kernel("append", lambda: [mk.window_append(projp[:, :p0.split], *c[0].get_kv_cache(), a.q_norm, a.k_norm, a.cos_sin, positions,
                                                           params.new_cache_slots, heads=heads, dim=128, off_q=0, off_k=a.off_k, off_v=a.off_v,
                                                           eps=1e-5) for x, c in paras], len(paras), nbytes=bs * 4 * (heads + 2 * kv_heads) * 128, bs=bs)
                seen = min(context, window + KEEP)
                kernel("decode attention", lambda: [mk.window_attention(
                    projp, *c[0].get_kv_cache(), out, a.sink, positions, params.q_cu_seq_lens, params.block_tables, params.cu_block_lens, heads=heads,
                    block_size=BLOCK, window=window, keep_first=KEEP, scale=0.09, softcap=30.0, max_kv_len=context) for x, c in paras], len(paras),
                    nbytes=bs * seen * kv_heads * 512, flops=4 * bs * seen * heads * 128, bs=bs)
                act = torch.randn(bs, ff, device=DEV).to(torch.bfloat16)
                wide = bs > lk.STREAM_MAX_ROWS

                def mm(name, fn, w, n):
                    kernel(name, fn, n, nbytes=w.numel() * 2, flops=2 * bs * w.numel(), bs=bs)
                mm("delta proj", lambda: [lk.linear(h, x.mixer.w_in) for x, _ in deltas], d0.w_in, len(deltas))
                mm("low-rank", lambda: [lk.linear_heads(projd[:, d0.off_a1:], d0.low_k, x.mixer.w_low, low, d0.low_n) for x, _ in deltas], d0.w_low,
                   len(deltas))
                mm("parallel proj", lambda: [lk.linear(h, x.mixer.w_in) for x, _ in paras], p0.w_in, len(paras))
                mm("gate_up+act", lambda: [lk.linear_glu(h, x.mlp.w_gate_up, act, float("inf"), 1.0, 0.0) for x in m.layers], m.layers[0].mlp.w_gate_up, L)
                mm("down", lambda: [(lk.linear if wide else lk.linear_slabs)(act, x.mlp.w_down) for x in m.layers], m.layers[0].mlp.w_down, L)
            for name, q_lens, kv_lens in cases:
                tokens, positions, params, _ = batch(q_lens, kv_lens, block, vocab, which != "llama")
                T = tokens.numel()
                if V:
                    params = with_states(params)
                if which == "llama":
                    m.reserve_workspaces(T, max(kv_lens))
                t = timed(lambda: m.forward(tokens, positions, params), graph=False)
                emit(kind="prefill", **base, batch=name, tokens=T, ms=t * 1e3, us_per_layer=t / L * 1e6, tokens_per_s=T / t)
                if not V:
                    continue
                projd = torch.randn(T, d0.w_in.size(0), device=DEV).to(torch.bfloat16)
                projp = torch.randn(T, p0.w_in.size(0), device=DEV).to(torch.bfloat16)
                low = torch.randn(T, 2 * d0.low_n, device=DEV).to(torch.bfloat16)
                out = torch.empty(T, max(p0.o_k, d0.o_k), device=DEV, dtype=torch.bfloat16)
                step = (positions, params.q_cu_seq_lens, params.state_slots, 0)
                chunks = mk.ChunkPlan.of(params, 0, DEV)
                x, c = deltas[0]
                # 32-bit products of a token in chunks of 16: three with the state, four 16 wide
                kernel("delta portions (prepare + scan)", lambda: mk.recurrent_portions(x.mixer.spec, projd, low, c, *step, chunks), 1, fp32=T * chunk_flops,
                       nbytes=T * heads * 128 * (8 + 4 * 8), batch=name)
                y, e = paras[0]
                kernel("lightning portions (prepare + scan)", lambda: mk.recurrent_portions(y.mixer.right.spec, projp[:, p0.split:], None, e[1], *step, chunks), 1,
                       fp32=T * (chunk_flops - 2 * S - 2 * heads * 2 * 16 * 128), nbytes=T * heads * 128 * (6 + 4 * 6), batch=name)
                o = torch.randn(T, heads, 128, device=DEV)
                kernel("norm + gate", lambda: mk.gated_norm(o, 128, low[:, d0.low_n:], d0.spec.norm_weight, out[:, :d0.o_k], eps=1e-5, per_head=True), 1,
                       nbytes=T * heads * 128 * 8, batch=name)
                a = p0.left
                plan = WindowPlan.of(params, window, KEEP, BLOCK, DEV)
                flops = 4 * heads * 128 * visible_pairs(q_lens, kv_lens, window)
                kernel("prompt attention", lambda: mk.window_prefill(projp, *e[0].get_kv_cache(), out, a.sink, plan.slots, plan.tiles, heads=heads,
                                                                     window=window, keep_first=KEEP, scale=0.09, softcap=30.0), 1, flops=flops, batch=name)
                kernel("append", lambda: mk.window_append(projp[:, :p0.split], *e[0].get_kv_cache(), a.q_norm, a.k_norm, a.cos_sin, positions,
                                                          params.new_cache_slots, heads=heads, dim=128, off_q=0, off_k=a.off_k, off_v=a.off_v, eps=1e-5),
                       1, nbytes=T * 4 * (heads + 2 * kv_heads) * 128, batch=name)
                h = torch.randn(T, m.k_width, device=DEV).to(torch.bfloat16)
                act = torch.empty(T, ff, device=DEV, dtype=torch.bfloat16)
                kernel("gate_up+act", lambda: [lk.linear_glu(h, z.mlp.w_gate_up, act, float("inf"), 1.0, 0.0) for z in m.layers], L, flops=4 * T * width * ff,
                       batch=name)
            del m
    return 0


if __name__ == "__main__":
    sys.exit(main())
