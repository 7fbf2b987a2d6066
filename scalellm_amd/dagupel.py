"""Dagupel: a small decoder-only model of windowed latent attention and clamped GLU feed-forwards over an fp32
residual stream, with learned positions and layers that may share another layer's weights.

The step function is the framework's: forward(tokens, positions, InputParameters) over a paged cache, driven by
ModelRunner (graphs for decode batches) and engine.LLMEngine.  Launches of a decode layer: projection, append
(latent norm + rotation + cache write), absorbed query product, attention (+ merge of its splits), value product with
the output gate, output projection (split-K slabs), add + norm, gate_up with the activation, down (slabs), add + norm.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Callable, List, Optional

import torch

from . import latent_kernels as lk
from .checkpoint import Checkpoint
from .kernels import SlmError, reserve_workspace
from .latent_layers import ClampedGLU, LatentAttention, LatentAttentionArgs, YarnScaling, rotary_table, round_up
from .layers import InputParameters
from .registry import ModelLimits, register_model


@dataclass
class DenseMLPArgs:
    ff: int
    limit: float


@dataclass
class DagupelLayer:
    mixer: LatentAttentionArgs
    mlp: Optional[DenseMLPArgs]
    weights_of: Optional[int]   # the layer whose tensors it uses


@dataclass
class DagupelConfig:
    vocab: int
    width: int
    max_positions: int
    eps: float
    logit_scale: float
    layers: List[DagupelLayer]

    @staticmethod
    def parse(c: dict) -> "DagupelConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            if e["type"] != "latent_attention":
                raise ValueError(f"layer {i}: unknown mixer {e['type']!r}")
            m, rot = e["mixer"], e["mixer"]["rot"]
            if rot["dims"] != m["rot_dim"] or m["rot_dim"] % 2:
                raise ValueError(f"layer {i}: rot.dims {rot['dims']} is not the rotated width {m['rot_dim']}")
            s = rot.get("scaling")
            mixer = LatentAttentionArgs(
                heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"], kv_rank=m["kv_rank"],
                scale=m["scale"], window=(m.get("mask") or {}).get("size") or 0, rot_base=rot["base"],
                rot_scaling=YarnScaling(s["factor"], s["original"], s["fast"], s["slow"]) if s else None)
            mlp = e.get("mlp")
            if mlp is not None:
                if mlp["kind"] != "dense":
                    raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
                mlp = DenseMLPArgs(ff=mlp["ff"], limit=mlp["limit"])
            j = e.get("weights_of")
            if j is not None and not 0 <= j < len(c["layers"]):
                raise ValueError(f"layer {i}: weights_of {j}")
            layers.append(DagupelLayer(mixer, mlp, j))
        return DagupelConfig(c["vocab"], c["width"], c["max_positions"], c["norm"]["eps"], c["logit_scale"], layers)

    def weight_layer(self, i: int) -> int:
        """The layer whose tensors layer i runs on."""
        seen = set()
        while self.layers[i].weights_of is not None:
            if i in seen:
                raise ValueError(f"layer {i}: weights_of goes round in a circle")
            seen.add(i)
            i = self.layers[i].weights_of
        return i


class _LayerWeights:
    __slots__ = ("attn", "mlp", "norm1", "norm2")


@register_model("Dagupel")
class DagupelStep:
    libraries = ("latent",)

    def __init__(self, config: DagupelConfig, ckpt: Checkpoint, limits: ModelLimits):
        c = self.config = config
        if limits.dtype not in (torch.bfloat16, torch.float32):
            raise SlmError(f"Dagupel runs in bfloat16 or float32, not {limits.dtype}")
        if limits.dtype == torch.float32 and torch.backends.cuda.matmul.allow_tf32:
            raise SlmError("float32 means true 32-bit: switch torch.backends.cuda.matmul.allow_tf32 off")
        self.dtype, self.device = limits.dtype, torch.device(limits.device)
        self.block_size = limits.block_size
        self.max_positions, self.vocab = c.max_positions, c.vocab
        dev, dt, W = self.device, self.dtype, c.width
        self.k_width = round_up(W, 64)
        # embedding and vocabulary projection are one table: zero padded to the product's tiles
        self.table = torch.zeros(round_up(c.vocab, 16), self.k_width, dtype=dt, device=dev)
        self.table[:c.vocab, :W] = ckpt.take("embed", (c.vocab, W)).to(device=dev, dtype=dt)
        self.pos_table = ckpt.take("pos", (c.max_positions, W)).to(device=dev, dtype=dt).contiguous()
        norm = lambda name: ckpt.take(name, (W,)).to(device=dev, dtype=torch.float32).contiguous()  # noqa: E731
        self.final_norm = norm("final.norm")
        tables, weights = {}, {}
        self.layers, self.caches = [], []
        for i in range(len(c.layers)):
            j = c.weight_layer(i)
            m, mlp = c.layers[j].mixer, c.layers[j].mlp
            if (c.layers[i].mixer, c.layers[i].mlp) != (m, mlp):
                raise ValueError(f"layer {i} differs from layer {j}, whose weights it uses")
            if j not in weights:
                L = weights[j] = _LayerWeights()
                p = f"l{j}."
                shapes = {"q": (m.heads * (m.dim + m.rot_dim), W), "dkv": (m.kv_rank + m.rot_dim, W), "dkv.norm": (m.kv_rank,),
                          "uk": (m.heads * m.dim, m.kv_rank), "uv": (m.heads * m.vdim, m.kv_rank), "g": (m.heads, W),
                          "o": (W, m.heads * m.vdim)}
                key = (m.rot_base, m.rot_dim, repr(m.rot_scaling))
                if key not in tables:
                    tables[key] = rotary_table(m.rot_base, m.rot_dim, c.max_positions, m.rot_scaling, dev)
                L.attn = LatentAttention(m, W, c.eps, {n: ckpt.take(p + "mix." + n, s) for n, s in shapes.items()}, tables[key],
                                         dt, dev)
                L.norm1, L.norm2, L.mlp = norm(p + "norm1"), None, None
                if mlp is not None:
                    L.norm2 = norm(p + "norm2")
                    L.mlp = ClampedGLU(W, mlp.ff, mlp.limit, {"gate": ckpt.take(p + "mlp.gate", (mlp.ff, W)),
                                                              "up": ckpt.take(p + "mlp.up", (mlp.ff, W)),
                                                              "down": ckpt.take(p + "mlp.down", (W, mlp.ff))}, dt, dev)
            self.layers.append(weights[j])
            self.caches.append(weights[j].attn.new_cache(limits.n_blocks, limits.block_size))
        # portions go to their own kernels where every layer has them (the step's rows are ordered once)
        self.portion_min = LatentAttention.PORTION_MIN if all(L.attn.portions_ok for L in self.layers) else None
        # called with (layer run, residual stream) after every layer, when set
        self.on_layer: Optional[Callable[[int, torch.Tensor], None]] = None

    @classmethod
    def from_checkpoint(cls, config: dict, ckpt: Checkpoint, limits: ModelLimits) -> "DagupelStep":
        model = cls(DagupelConfig.parse(config), ckpt, limits)
        ckpt.finish()
        return model

    def reserve_workspaces(self, n_tokens: int) -> None:
        """Size the attention scratch for decode batches of up to n_tokens rows, before graphs are captured."""
        need = max(n_tokens, 512) * max(L.attn.args.heads * (L.attn.c_pad + 2) for L in self.layers) * 4
        reserve_workspace(2 * need, self.device)

    def forward(self, tokens: torch.Tensor, positions: torch.Tensor, params: InputParameters,
                return_logits: bool = False) -> torch.Tensor:
        """One step: tokens / positions [T] int32 -> logits [wanted rows, vocab] fp32, or their arg max (greedy ids).
        Wanted rows: params.logit_rows, by default the last row of every sequence."""
        c, T = self.config, tokens.numel()
        resid = torch.empty(T, c.width, dtype=torch.float32, device=self.device)
        h = torch.empty(T, self.k_width, dtype=self.dtype, device=self.device)
        first = self.layers[0].norm1 if self.layers else None
        lk.residual_norm(resid, h, first, c.eps, embed=(tokens, self.table, positions, self.pos_table))
        n = len(self.layers)
        for i, L in enumerate(self.layers):
            nxt = self.layers[i + 1].norm1 if i + 1 < n else None
            delta = L.attn.forward(h, positions, self.caches[i], params)
            if L.mlp is not None:
                lk.residual_norm(resid, h, L.norm2, c.eps, delta=delta)
                delta = L.mlp.forward(h)
            lk.residual_norm(resid, h, nxt, c.eps, delta=delta)
            if self.on_layer is not None:
                self.on_layer(i, resid)
        rows = params.logit_rows
        if rows is None:
            rows = params.q_cu_seq_lens[1:] - 1
        out = torch.empty(rows.numel(), self.k_width, dtype=self.dtype, device=self.device)
        if rows.numel() == 0:
            return torch.empty(0, c.vocab, dtype=torch.float32, device=self.device)
        lk.residual_norm(resid, out, self.final_norm, c.eps, row_index=rows)
        logits = lk.linear_f32(out, self.table, c.logit_scale)[:, :c.vocab]
        if return_logits:
            return logits
        return torch.argmax(logits, dim=-1).to(torch.int32)
