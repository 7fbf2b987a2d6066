"""Plain, slow restatement of the Dagupel design in double precision (numpy): one function per mechanism, no cache, no
batch, no padding.  Checker only; shares no code with scalellm_amd."""
from __future__ import annotations

import math

import numpy as np


def rms_norm(x, weight, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def yarn_frequencies(rot):
    """(frequency per pair, factor of cos and sin) of a rotation {base, dims, scaling?}."""
    d, base = rot["dims"], rot["base"]
    freqs, magnitude = [], 1.0
    s = rot.get("scaling")
    for i in range(d // 2):
        f = base ** (-2.0 * i / d)
        if s:
            def where(turns):
                return d * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
            lo, hi = max(math.floor(where(s["fast"])), 0), min(math.ceil(where(s["slow"])), d - 1)
            ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
            f = f / s["factor"] * ramp + f * (1.0 - ramp)
        freqs.append(f)
    if s:
        magnitude = 0.1 * math.log(s["factor"]) + 1.0
    return np.array(freqs), magnitude


def rotate(x, positions, rot):
    """x [tokens, ..., dims]: pairs (i, i + dims / 2) turned by position * frequency."""
    freqs, magnitude = yarn_frequencies(rot)
    half = rot["dims"] // 2
    out = np.array(x)
    for t, p in enumerate(positions):
        c, s = np.cos(p * freqs) * magnitude, np.sin(p * freqs) * magnitude
        u, v = x[t, ..., :half], x[t, ..., half:]
        out[t, ..., :half], out[t, ..., half:] = u * c - v * s, v * c + u * s
    return out


def visible(i, window):
    """Positions token i attends to."""
    return range(max(0, i - window + 1) if window else 0, i + 1)


def latent_attention(h, w, m, eps, first=0):
    """The mixer over a whole sequence: h [tokens, width] -> [tokens, width].  w: tensors by their short names."""
    n, H = h.shape[0], m["heads"]
    D, Rd, V, K = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    positions = range(first, first + n)
    q = (h @ w["q"].T).reshape(n, H, D + Rd)
    q_rot = rotate(q[:, :, D:], positions, m["rot"])
    down = h @ w["dkv"].T
    c = rms_norm(down[:, :K], w["dkv.norm"], eps)
    k_rot = rotate(down[:, K:], positions, m["rot"])
    k, v = (c @ w["uk"].T).reshape(n, H, D), (c @ w["uv"].T).reshape(n, H, V)
    gate = sigmoid(h @ w["g"].T)
    window = (m.get("mask") or {}).get("size") or 0
    out = np.zeros((n, H, V))
    for i in range(n):
        js = list(visible(i, window))
        for head in range(H):
            s = (k[js, head] @ q[i, head, :D] + k_rot[js] @ q_rot[i, head]) * m["scale"]
            p = np.exp(s - s.max())
            out[i, head] = (p / p.sum()) @ v[js, head] * gate[i, head]
    return out.reshape(n, H * V) @ w["o"].T


def clamped_glu(gate, up, limit):
    g, u = np.minimum(gate, limit), np.clip(up, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def feed_forward(h, w, mlp):
    return clamped_glu(h @ w["gate"].T, h @ w["up"].T, mlp["limit"]) @ w["down"].T


def weight_layer(config, i):
    while config["layers"][i].get("weights_of") is not None:
        i = config["layers"][i]["weights_of"]
    return i


def forward(config, tensors, tokens, residuals=None):
    """Logits [tokens, vocab] of one sequence.  tensors: name -> float64 array.  residuals: list that receives the
    residual stream after every layer."""
    eps = config["norm"]["eps"]
    x = tensors["embed"][tokens] + tensors["pos"][np.arange(len(tokens))]
    for i, layer in enumerate(config["layers"]):
        pre = f"l{weight_layer(config, i)}."
        w = {k[len(pre) + 4:]: v for k, v in tensors.items() if k.startswith((pre + "mix.", pre + "mlp."))}
        x = x + latent_attention(rms_norm(x, tensors[pre + "norm1"], eps), w, layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + feed_forward(rms_norm(x, tensors[pre + "norm2"], eps), w, layer["mlp"])
        if residuals is not None:
            residuals.append(x)
    return rms_norm(x, tensors["final.norm"], eps) @ tensors["embed"].T * config["logit_scale"]
