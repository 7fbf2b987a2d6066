"""Vebusun: a small decoder-only model whose layers mix tokens by a gated delta rule with a decay per key channel, or by
windowed attention and lightning attention side by side; SiLU GLU feed-forwards, tanh norms, an fp32 residual stream, and
a range of layers that runs several times with the same weights.

The step function is the framework's: forward(tokens, positions, InputParameters) over a paged cache and per-sequence
state slots, driven by ModelRunner (graphs for decode batches) and engine.LLMEngine.  Every pass of a looped layer has a
cache or state of its own.  Launches of a decode layer: delta -- projection, low-rank products, recurrence (convolution,
gates, update, norm and gate), output projection (split-K slabs), add + norm; parallel -- projection, append (norms,
rotation, cache write), attention (+ merge of its splits), recurrence, norm + gate, output projection, add + norm;
feed-forward -- gate_up with the activation, down (slabs), add + norm.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Callable, List, Optional, Union

import torch

from . import latent_kernels as lk
from .checkpoint import Checkpoint
from .kernels import SlmError, reserve_workspace
from .latent_layers import ClampedGLU, rotary_table, round_up
from .layers import InputParameters
from .mixer_layers import (ChannelDelta, ChannelDeltaArgs, LightningArgs, LightningAttention, ParallelMixer, WindowAttention,
                           WindowAttentionArgs)
from .registry import ModelLimits, register_model


@dataclass
class ParallelArgs:
    left: WindowAttentionArgs
    right: LightningArgs
    left_scale: float
    right_scale: float


@dataclass
class VebusunLayer:
    mixer: Union[ChannelDeltaArgs, ParallelArgs]
    ff: Optional[int]    # width of the feed-forward; None = no feed-forward


def _parse_mixer(i: int, e: dict):
    m = e["mixer"]
    if e["type"] == "channel_delta":
        return ChannelDeltaArgs(heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"], vdim=m["vdim"], taps=m["conv"])
    if e["type"] != "parallel":
        raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
    a, b = m["left"], m["right"]
    rot, mask = a.get("rot") or {"base": 1.0, "dims": 0}, a.get("mask") or {}
    if rot["dims"] % 2 or rot["dims"] > a["dim"]:
        raise ValueError(f"layer {i}: {rot['dims']} rotated dimensions of {a['dim']}")
    left = WindowAttentionArgs(heads=a["heads"], kv_heads=a["kv_heads"], dim=a["dim"], vdim=a["vdim"], scale=a["scale"],
                               rot_base=rot["base"], rot_dims=rot["dims"], softcap=a.get("softcap") or 0.0,
                               window=mask.get("size") or 0, keep_first=mask.get("keep_first") or 0)
    right = LightningArgs(heads=b["heads"], dim=b["dim"], vdim=b["vdim"], decay=[float(d) for d in b["decay"]])
    return ParallelArgs(left, right, m["left_scale"], m["right_scale"])


@dataclass
class VebusunConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    residual_mult: float
    layers: List[VebusunLayer]
    runs: List[int]      # layer indexes in the order they run

    @staticmethod
    def parse(c: dict) -> "VebusunConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            mlp = e.get("mlp")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            layers.append(VebusunLayer(_parse_mixer(i, e), mlp["ff"] if mlp is not None else None))
        n, loop = len(layers), c.get("loop")
        runs = list(range(n))
        if loop is not None:
            a, b, times = loop["start"], loop["stop"], loop["times"]
            if not 0 <= a <= b <= n or times < 0:
                raise ValueError(f"loop over layers {a} .. {b}, {times} times, of {n}")
            runs = runs[:a] + runs[a:b] * times + runs[b:]
        return VebusunConfig(c["vocab"], c["width"], c["norm"]["eps"], c["embedding"]["scale"], c["residual_mult"], layers, runs)


class _LayerWeights:
    __slots__ = ("mixer", "mlp", "norm1", "norm2")


@register_model("Vebusun")
class VebusunStep:
    libraries = ("latent", "mixers")
    portion_min = 2   # (a recurrence runs over whole portions)

    def __init__(self, config: VebusunConfig, ckpt: Checkpoint, limits: ModelLimits):
        c = self.config = config
        if limits.dtype not in (torch.bfloat16, torch.float32):
            raise SlmError(f"Vebusun runs in bfloat16 or float32, not {limits.dtype}")
        self.dtype, self.device = limits.dtype, torch.device(limits.device)
        self.block_size, self.vocab, self.n_states = limits.block_size, c.vocab, limits.n_states
        self.max_positions = limits.max_positions or limits.n_blocks * limits.block_size
        dev, dt, W = self.device, self.dtype, c.width
        self.k_width = round_up(W, 64)
        self.embed = ckpt.take("embed", (c.vocab, W)).to(device=dev, dtype=dt).contiguous()
        self.head = torch.zeros(round_up(c.vocab, 16), self.k_width, dtype=dt, device=dev)
        self.head[:c.vocab, :W] = ckpt.take("head", (c.vocab, W)).to(device=dev, dtype=dt)
        f32 = lambda name: ckpt.take(name, (W,)).to(device=dev, dtype=torch.float32).contiguous()  # noqa: E731

        def norm(name):
            return lk.TanhNorm(ckpt.take(name + ".alpha").float().item(), f32(name), f32(name + ".b"))   # (a scalar)
        self.final_norm = norm("final.norm")
        tables = {}

        def rotation(a: WindowAttentionArgs):
            key = (a.rot_base, a.rot_dims)
            if key not in tables:
                tables[key] = rotary_table(a.rot_base, a.rot_dims, self.max_positions, device=dev)
            return tables[key]

        weights = []
        for i, layer in enumerate(c.layers):
            L, p = _LayerWeights(), f"l{i}."
            L.mixer = self._mixer(layer.mixer, p + "mix.", ckpt, rotation)
            L.norm1, L.norm2, L.mlp = norm(p + "norm1"), None, None
            if layer.ff is not None:
                L.norm2 = norm(p + "norm2")
                L.mlp = ClampedGLU(W, layer.ff, math.inf, {"gate": ckpt.take(p + "mlp.gate", (layer.ff, W)),
                                                           "up": ckpt.take(p + "mlp.up", (layer.ff, W)),
                                                           "down": ckpt.take(p + "mlp.down", (W, layer.ff))}, dt, dev, 1.0, 0.0)
            elif p + "norm2" in ckpt.names():   # (a norm nothing follows)
                norm(p + "norm2")
            weights.append(L)
        self.layers = [weights[i] for i in c.runs]
        self.caches = [L.mixer.new_cache(limits) for L in self.layers]
        # called with (layer run, residual stream) after every layer, when set
        self.on_layer: Optional[Callable[[int, torch.Tensor], None]] = None

    def _mixer(self, m, p: str, ckpt: Checkpoint, rotation):
        c, W, dt, dev = self.config, self.config.width, self.dtype, self.device
        if isinstance(m, ChannelDeltaArgs):
            H, G, D, V = m.heads, m.kv_heads, m.dim, m.vdim
            shapes = {"q": (G * D, W), "k": (G * D, W), "v": (H * V, W), "q.conv": (G * D, m.taps), "k.conv": (G * D, m.taps),
                      "v.conv": (H * V, m.taps), "b": (H, W), "A_log": (H,), "dt_bias": (H * D,), "norm": (V,), "o": (W, H * V)}
            w = {n: ckpt.take(p + n, s) for n, s in shapes.items()}
            for first, second, n in (("a1", "a2", H * D), ("g1", "g2", H * V)):   # (the rank is the tensors' own)
                w[first] = ckpt.take(p + first)
                if w[first].dim() != 2 or w[first].size(1) != W:
                    raise ValueError(f"{p}{first}: shape {tuple(w[first].shape)}")
                w[second] = ckpt.take(p + second, (n, w[first].size(0)))
            return ChannelDelta(m, W, c.eps, w, dt, dev)
        a, b = m.left, m.right
        left = {"q": (a.heads * a.dim, W), "k": (a.kv_heads * a.dim, W), "v": (a.kv_heads * a.vdim, W), "q.norm": (a.dim,),
                "k.norm": (a.dim,), "sink": (a.heads,), "o": (W, a.heads * a.vdim)}
        qk, vo = b.heads * b.dim, b.heads * b.vdim
        right = {"q": (qk, W), "k": (qk, W), "v": (vo, W), "g": (vo, W), "norm": (vo,), "o": (W, vo)}
        left = {n: ckpt.take(f"{p}left.{n}", s) for n, s in left.items()}
        right = {n: ckpt.take(f"{p}right.{n}", s) for n, s in right.items()}
        return ParallelMixer(WindowAttention(a, W, c.eps, left, rotation(a), dt, dev, m.left_scale),
                             LightningAttention(b, W, c.eps, right, dt, dev, m.right_scale), W)

    @classmethod
    def from_checkpoint(cls, config: dict, ckpt: Checkpoint, limits: ModelLimits) -> "VebusunStep":
        model = cls(VebusunConfig.parse(config), ckpt, limits)
        ckpt.finish()
        return model

    def reserve_workspaces(self, n_tokens: int) -> None:
        """Size the attention scratch for decode batches of up to n_tokens rows, before graphs are captured."""
        need = [L.mixer.left.args.heads * (L.mixer.left.v_pad + 2) * 4 for L in self.layers if isinstance(L.mixer, ParallelMixer)]
        if need:   # (a split per spare workgroup: no more than about 1024 workgroups' worth of rows)
            reserve_workspace(2 * max(n_tokens, 1024) * max(need), self.device)

    def forward(self, tokens: torch.Tensor, positions: torch.Tensor, params: InputParameters,
                return_logits: bool = False) -> torch.Tensor:
        """One step: tokens / positions [T] int32 -> logits [wanted rows, vocab] fp32, or their arg max (greedy ids).
        Wanted rows: params.logit_rows, by default the last row of every sequence."""
        c, T = self.config, tokens.numel()
        resid = torch.empty(T, c.width, dtype=torch.float32, device=self.device)
        h = torch.empty(T, self.k_width, dtype=self.dtype, device=self.device)
        n = len(self.layers)
        lk.residual_norm(resid, h, self.layers[0].norm1 if n else None, c.eps, embed=(tokens, self.embed, None, None), mult=c.embedding_scale)
        for i, L in enumerate(self.layers):
            nxt = self.layers[i + 1].norm1 if i + 1 < n else None
            delta = L.mixer.forward(h, positions, self.caches[i], params)
            if L.mlp is not None:
                lk.residual_norm(resid, h, L.norm2, c.eps, delta=delta, mult=c.residual_mult)
                delta = L.mlp.forward(h)
            lk.residual_norm(resid, h, nxt, c.eps, delta=delta, mult=c.residual_mult)
            if self.on_layer is not None:
                self.on_layer(i, resid)
        rows = params.logit_rows
        if rows is None:
            rows = params.q_cu_seq_lens[1:] - 1
        if rows.numel() == 0:
            return torch.empty(0, c.vocab, dtype=torch.float32, device=self.device)
        out = torch.empty(rows.numel(), self.k_width, dtype=self.dtype, device=self.device)
        lk.residual_norm(resid, out, self.final_norm, c.eps, row_index=rows)
        logits = lk.linear_f32(out, self.head)[:, :c.vocab]
        return logits if return_logits else torch.argmax(logits, dim=-1).to(torch.int32)
