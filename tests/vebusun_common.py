"""Small random Vebusun models for the tests: configurations and weights."""
from __future__ import annotations

import torch

from .dagupel_common import as_f64, row_errors, write_model  # noqa: F401


def delta(heads, kv_heads, dim, vdim, conv):
    return "channel_delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def parallel(left, right, left_scale=1.0, right_scale=1.0):
    return "parallel", {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def window(heads, kv_heads, dim, vdim, rot_dims, size, keep, softcap=30.0, scale=None, base=10000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": rot_dims},
            "mask": {"size": size, "keep_first": keep}, "scale": scale if scale is not None else dim ** -0.5, "softcap": softcap}


def lightning(dim, vdim, decay):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def config(width, layers, vocab=90, eps=1e-5, embedding_scale=2.0, residual_mult=0.5, loop=None):
    """layers: ((type, mixer), ff or None); loop: (start, stop, times)."""
    return {"architecture": "Vebusun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embedding_scale},
            "residual_mult": residual_mult, "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop)),
            "layers": [{"type": kind, "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
                       for (kind, m), ff in layers]}


def mixer_weights(kind, m, width, rnd, rank=9, sharp=1.0):
    """Tensors of one mixer by their short names.  sharp > 1 scales the query norm: soft-max weights then rest on few keys."""
    W, s = width, width ** -0.5
    if kind == "channel_delta":
        qk, H, vo = m["kv_heads"] * m["dim"], m["heads"], m["heads"] * m["vdim"]
        t = {}
        for n, c in (("q", qk), ("k", qk), ("v", vo)):
            t[n], t[n + ".conv"] = rnd(c, W, std=2 * s), rnd(c, m["conv"], std=0.6)
        t.update({"b": rnd(H, W, std=2 * s), "A_log": rnd(H, mean=-1.0), "a1": rnd(rank, W, std=s), "a2": rnd(H * m["dim"], rank, std=rank ** -0.5),
                  "dt_bias": rnd(H * m["dim"], mean=-2.0), "g1": rnd(rank + 4, W, std=s), "g2": rnd(vo, rank + 4, std=(rank + 4) ** -0.5),
                  "norm": rnd(m["vdim"], std=0.2, mean=1.0), "o": rnd(W, vo, std=2 * vo ** -0.5)})
        return t
    a, b = m["left"], m["right"]
    H, G, D, V = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
    qk, vo = b["heads"] * b["dim"], b["heads"] * b["vdim"]
    return {"left.q": rnd(H * D, W, std=s), "left.k": rnd(G * D, W, std=s), "left.v": rnd(G * V, W, std=s),
            "left.q.norm": rnd(D, std=0.2, mean=sharp), "left.k.norm": rnd(D, std=0.2, mean=1.0), "left.sink": rnd(H, mean=1.0),
            "left.o": rnd(W, H * V, std=2 * (H * V) ** -0.5),
            "right.q": rnd(qk, W, std=2 * s), "right.k": rnd(qk, W, std=2 * s), "right.v": rnd(vo, W, std=2 * s), "right.g": rnd(vo, W, std=2 * s),
            "right.norm": rnd(vo, std=0.2, mean=1.0), "right.o": rnd(W, vo, std=2 * vo ** -0.5)}


def random_tensors(seed):
    g = torch.Generator().manual_seed(seed)

    def rnd(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16)
    return rnd


def weights(cfg, seed, sharp=2.0):
    rnd, W = random_tensors(seed), cfg["width"]
    t = {"embed": rnd(cfg["vocab"], W), "head": rnd(cfg["vocab"], W, std=W ** -0.5)}

    def norm(name):
        t[name], t[name + ".b"] = rnd(W, std=0.3, mean=1.0), rnd(W, std=0.1)
        t[name + ".alpha"] = rnd(1, std=0.1, mean=0.6).view(())
    norm("final.norm")
    for i, e in enumerate(cfg["layers"]):
        p = f"l{i}."
        norm(p + "norm1")
        t.update({p + "mix." + n: x for n, x in mixer_weights(e["type"], e["mixer"], W, rnd, rank=5 + 3 * i, sharp=sharp).items()})
        if e["mlp"] is not None:
            norm(p + "norm2")
            ff = e["mlp"]["ff"]
            t[p + "mlp.gate"], t[p + "mlp.up"] = rnd(ff, W, std=2 * W ** -0.5), rnd(ff, W, std=W ** -0.5)
            t[p + "mlp.down"] = rnd(W, ff, std=2 * ff ** -0.5)
    return t


CONFIGS = {
    # nothing is a multiple of a tile; grouped heads in both mixers; the loop starts and ends inside; a layer without feed-forward
    "odd": config(77, [(delta(4, 2, 20, 13, 3), 51), (parallel(window(6, 3, 22, 18, 10, 21, 5, 5.0), lightning(11, 7, (0.5, 0.9, 0.99)), 0.7, 1.3), None),
                       (delta(3, 1, 9, 33, 4), 40)], vocab=93, loop=(1, 3, 3)),
    # one head, a window of one token, nothing kept, a convolution of one tap, values of one column; no loop
    "tiny": config(32, [(delta(1, 1, 8, 1, 1), None), (parallel(window(1, 1, 8, 4, 8, 1, 0, 2.0, 1.0), lightning(3, 5, (0.8,))), 16)], vocab=17,
                   residual_mult=1.0, embedding_scale=1.0),
    # more query heads on a key head than one block, wide values, kept tokens beyond a key tile; a loop over everything
    "wide": config(128, [(parallel(window(40, 2, 128, 96, 64, 70, 67, 12.0, base=500.0), lightning(64, 128, (0.7, 0.999)), 0.4, 0.6), 64),
                         (delta(3, 3, 100, 150, 5), 96)], vocab=160, eps=1e-3, loop=(0, 2, 2)),
    # sizes only the any-size attention has, the widest states, no window; a loop of one pass
    "large": config(64, [(delta(2, 2, 200, 256, 2), None), (parallel(window(2, 1, 260, 300, 60, 0, 0, 0.0), lightning(130, 200, (0.95, 0.99))), 48)],
                    vocab=48, loop=(0, 1, 1)),
}
