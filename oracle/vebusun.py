"""Plain, slow restatement of the Vebusun design in double precision (numpy): one function per mechanism, no cache, no
batch, no padding, one token after the other where a recurrence runs.  For tests only; shares no code with scalellm_amd."""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rms_norm(x, weight, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * weight


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def dynamic_tanh(x, alpha, weight, bias):
    return np.tanh(alpha * x) * weight + bias


def rotate(x, positions, base, dims):
    """x [tokens, heads, width]: pairs (i, i + dims / 2) of the first `dims` entries turned by position * base^(-2 i / dims)."""
    out = np.array(x)
    half = dims // 2
    f = np.array([base ** (-2.0 * i / dims) for i in range(half)])
    for t, p in enumerate(positions):
        c, s = np.cos(p * f), np.sin(p * f)
        u, v = x[t, :, :half], x[t, :, half:dims]
        out[t, :, :half], out[t, :, half:dims] = u * c - v * s, v * c + u * s
    return out


def visible(i, mask):
    """Positions token i attends to: the last `size` and the first `keep_first`."""
    size, keep = (mask or {}).get("size") or 0, (mask or {}).get("keep_first") or 0
    return [j for j in range(i + 1) if not size or i - j < size or j < keep]


def sink_attention(h, w, m, eps):
    """Grouped heads, normed and rotated queries and keys, capped scores, a sink in the denominator."""
    n, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ w["q"].T).reshape(n, H, D), w["q.norm"], eps)
    k = rms_norm((h @ w["k"].T).reshape(n, G, D), w["k.norm"], eps)
    v = (h @ w["v"].T).reshape(n, G, V)
    q, k = (rotate(x, range(n), m["rot"]["base"], m["rot"]["dims"]) for x in (q, k))
    out = np.zeros((n, H, V))
    for i in range(n):
        js = visible(i, m.get("mask"))
        for a in range(H):
            g = a // (H // G)
            s = k[js, g] @ q[i, a] * m["scale"]
            if m.get("softcap"):
                s = m["softcap"] * np.tanh(s / m["softcap"])
            top = max(s.max(), w["sink"][a])
            p = np.exp(s - top)
            out[i, a] = p @ v[js, g] / (p.sum() + np.exp(w["sink"][a] - top))
    return out.reshape(n, H * V) @ w["o"].T


def lightning_recurrence(q, k, v, decay):
    """q, k [tokens, heads, dim], v [tokens, heads, vdim]: the read-outs of S <- decay S + k v^T."""
    state = np.zeros((q.shape[1], q.shape[2], v.shape[2]))
    out = np.zeros_like(v)
    for t in range(len(q)):
        state = np.asarray(decay)[:, None, None] * state + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hd,hdv->hv", q[t], state)
    return out


def lightning_attention(h, w, m, eps):
    n, H = len(h), m["heads"]
    q, k = (silu(h @ w[x].T).reshape(n, H, m["dim"]) for x in "qk")
    o = lightning_recurrence(q, k, silu(h @ w["v"].T).reshape(n, H, m["vdim"]), m["decay"])
    return (rms_norm(o.reshape(n, -1), w["norm"], eps) * sigmoid(h @ w["g"].T)) @ w["o"].T


def short_conv(x, taps):
    """x [tokens, channels], taps [channels, n]: the last tap meets the current token."""
    n = taps.shape[1]
    padded = np.concatenate([np.zeros((n - 1, x.shape[1])), x])
    return sum(padded[j:j + len(x)] * taps[:, j] for j in range(n))


def delta_recurrence(q, k, v, g, beta):
    """q, k, g [tokens, heads, dim], v [tokens, heads, vdim], beta [tokens, heads]."""
    state = np.zeros((q.shape[1], q.shape[2], v.shape[2]))
    out = np.zeros_like(v)
    for t in range(len(q)):
        state = state * g[t][:, :, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hd,hdv->hv", k[t], state))
        state = state + k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hd,hdv->hv", q[t], state)
    return out


def channel_delta(h, w, m, eps):
    n, H, G, D, V = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ w[x].T, w[x + ".conv"])) for x in "qkv")
    q, k = (np.repeat(unit(x.reshape(n, G, D)), H // G, axis=1) for x in (q, k))
    beta = sigmoid(h @ w["b"].T)
    step = softplus(h @ w["a1"].T @ w["a2"].T + w["dt_bias"]).reshape(n, H, D)
    g = np.exp(-np.exp(w["A_log"])[:, None] * step)
    o = delta_recurrence(q * D ** -0.5, k, v.reshape(n, H, V), g, beta)
    gate = sigmoid(h @ w["g1"].T @ w["g2"].T).reshape(n, H, V)
    return (rms_norm(o, w["norm"], eps) * gate).reshape(n, H * V) @ w["o"].T


def mixer(layer, h, w, eps):
    m = layer["mixer"]
    if layer["type"] == "channel_delta":
        return channel_delta(h, w, m, eps)
    left = {k[5:]: v for k, v in w.items() if k.startswith("left.")}
    right = {k[6:]: v for k, v in w.items() if k.startswith("right.")}
    return m["left_scale"] * sink_attention(h, left, m["left"], eps) + m["right_scale"] * lightning_attention(h, right, m["right"], eps)


def feed_forward(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def layer_runs(config):
    """Layer indexes in the order they run."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return list(range(n))
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(config, tensors, tokens, residuals=None):
    """Logits [tokens, vocab] of one sequence.  tensors: name -> float64 array.  residuals: list that receives the
    residual stream after every layer run."""
    eps, mult = config["norm"]["eps"], config["residual_mult"]

    def norm(x, name):
        return dynamic_tanh(x, tensors[name + ".alpha"], tensors[name], tensors[name + ".b"])
    x = tensors["embed"][np.asarray(tokens)] * config["embedding"]["scale"]
    for i in layer_runs(config):
        layer, pre = config["layers"][i], f"l{i}."
        w = {k[len(pre) + 4:]: v for k, v in tensors.items() if k.startswith((pre + "mix.", pre + "mlp."))}
        x = x + mult * mixer(layer, norm(x, pre + "norm1"), w, eps)
        if layer.get("mlp"):
            x = x + mult * feed_forward(norm(x, pre + "norm2"), w)
        if residuals is not None:
            residuals.append(x)
    return norm(x, "final.norm") @ tensors["head"].T
