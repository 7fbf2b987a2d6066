"""Small random Dagupel models for the tests: configurations, weights, a safetensors writer."""
from __future__ import annotations

import json
import os
import struct

import numpy as np
import torch


def mixer(heads, dim, rot_dim, vdim, kv_rank, window, scale=None, base=10000.0, scaling=None):
    rot = {"base": base, "dims": rot_dim}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": window},
            "scale": scale if scale is not None else (dim + rot_dim) ** -0.5, "rot": rot}


def config(width, layers, vocab=90, max_positions=512, eps=1e-5, logit_scale=1.0):
    """layers: (mixer, ff or None, limit) or an index whose weights are used again."""
    out = []
    for e in layers:
        if isinstance(e, int):
            j = e
            while "weights_of" in out[j]:
                j = out[j]["weights_of"]
            out.append(dict(out[j], weights_of=e))
        else:
            m, ff, limit = e
            out.append({"type": "latent_attention", "mixer": m,
                        "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}})
    return {"architecture": "Dagupel", "vocab": vocab, "width": width, "max_positions": max_positions, "norm": {"eps": eps},
            "logit_scale": logit_scale, "layers": out}


def weights(cfg, seed, sharp=1.0):
    """Random bf16 tensors.  sharp > 1 scales the queries: soft-max weights then rest on few keys, and one that is
    missing or extra shows."""
    g = torch.Generator().manual_seed(seed)
    W = cfg["width"]

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16)
    t = {"embed": rnd(cfg["vocab"], W), "pos": rnd(cfg["max_positions"], W, std=0.5), "final.norm": rnd(W, std=0.2, mean=1.0)}
    for i, e in enumerate(cfg["layers"]):
        if "weights_of" in e:
            continue
        m, p = e["mixer"], f"l{i}."
        H, D, R, V, K = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        t[p + "norm1"] = rnd(W, std=0.2, mean=1.0)
        t[p + "mix.q"] = rnd(H * (D + R), W, std=sharp * W ** -0.5)
        t[p + "mix.dkv"] = rnd(K + R, W, std=W ** -0.5)
        t[p + "mix.dkv.norm"] = rnd(K, std=0.2, mean=1.0)
        t[p + "mix.uk"] = rnd(H * D, K, std=K ** -0.5)
        t[p + "mix.uv"] = rnd(H * V, K, std=K ** -0.5)
        t[p + "mix.g"] = rnd(H, W, std=2 * W ** -0.5)
        t[p + "mix.o"] = rnd(W, H * V, std=2 * (H * V) ** -0.5)
        if e["mlp"] is not None:
            ff = e["mlp"]["ff"]
            t[p + "norm2"] = rnd(W, std=0.2, mean=1.0)
            t[p + "mlp.gate"] = rnd(ff, W, std=2 * W ** -0.5)
            t[p + "mlp.up"] = rnd(ff, W, std=2 * W ** -0.5)
            t[p + "mlp.down"] = rnd(W, ff, std=ff ** -0.5)
    return t


def as_f64(tensors):
    return {k: v.double().numpy() for k, v in tensors.items()}


def write_model(path, cfg, tensors):
    """config.json + model.safetensors in the folder `path`."""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    names = {torch.bfloat16: "BF16", torch.float32: "F32", torch.int32: "I32"}
    header, blobs, at = {}, [], 0
    for k, v in tensors.items():
        raw = v.contiguous().view(-1).view(torch.uint8).numpy().tobytes() if v.numel() else b""
        header[k] = {"dtype": names[v.dtype], "shape": list(v.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(header).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + b"".join(blobs))


def row_errors(got, want):
    """Root mean square difference per row, means taken off, over the root mean square of all of `want`."""
    d = np.asarray(got, dtype=np.float64) - want
    d -= d.mean(-1, keepdims=True)
    w = want - want.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((w * w).mean())


YARN = (4.0, 64, 8.0, 1.0)
# name -> (config, sharpness of the queries)
CONFIGS = {
    # nothing is a multiple of a tile: width, heads, every head part, rank, ff, vocabulary
    "odd": (config(77, [(mixer(3, 20, 6, 13, 37, 21, scaling=YARN), 51, 1.5), 0, (mixer(5, 9, 10, 7, 21, 33), None, 0)], vocab=93), 2.0),
    # one head, a window of one token, feed-forwards missing, sharing of a shared layer
    "tiny": (config(32, [(mixer(1, 32, 2, 32, 64, 1, scale=1.0), None, 0), (mixer(1, 8, 8, 1, 5, 2), 16, 0.5), 1, 2], vocab=17), 1.0),
    # head counts beyond one and two head blocks, two windows, wide latents, other norms and scales
    "wide": (config(128, [(mixer(20, 32, 64, 64, 100, 70, base=500.0, scaling=(2.0, 128, 16.0, 2.0)), 64, 3.0),
                          (mixer(40, 40, 34, 96, 200, 150, base=777.0), 192, 0.7)], vocab=160, eps=1e-3, logit_scale=0.125), 2.0),
    # no window, a rank beyond 256, values wider than queries, ramp of no width
    "deep": (config(96, [(mixer(4, 16, 32, 100, 300, 0, scaling=(8.0, 32, 1.0, 1.0)), 80, 1.0), 0, 0], vocab=64, logit_scale=2.0), 2.5),
    # sizes no fast kernel has: the any-size attention in 16 bits as well
    "large": (config(64, [(mixer(2, 250, 96, 160, 600, 40), 64, 1.0)], vocab=48), 2.0),
}
