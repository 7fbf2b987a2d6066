"""Layers of the dense 16- / 32-bit path over libslm_latent: rotary tables with YaRN scaling, the latent cache,
windowed latent attention with an output gate, and the clamped GLU feed-forward.

Weights come as plain tensors in checkpoint layout ([out, in]) and are laid out once at load: projections that read
the same input are merged into one product, heads are padded to the kernels' tile widths with zero rows, and W_uk is
kept in both forms a key can be met in (absorbed into the query for single tokens, expanded for prompt portions).
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence

import numpy as np
import torch

from . import _lib
from . import latent_kernels as lk
from .layers import InputParameters, Portion


def round_up(x: int, m: int) -> int:
    return (x + m - 1) // m * m


# ---------------------------------------------------------------------------------------
# rotary tables
# ---------------------------------------------------------------------------------------
@dataclass
class YarnScaling:
    """Context extension by parts: slow dimensions are interpolated by `factor`, fast ones kept, with a linear ramp
    between the dimensions that turn `fast` and `slow` times over `original` positions."""
    factor: float
    original: float
    fast: float
    slow: float


def rotary_table(base: float, dims: int, max_position: int, scaling: Optional[YarnScaling] = None, device="cpu") -> torch.Tensor:
    """[max_position, dims] = cos | sin, fp32 (computed in double): frequency of pair i = base^(-2 i / dims), scaled
    by parts with `scaling`, whose magnitude 0.1 ln(factor) + 1 is folded into both halves."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    freq = float(base) ** (-2.0 * i / dims)
    magnitude = 1.0
    if scaling is not None:
        def turns(t: float) -> float:
            return dims * math.log(scaling.original / (2.0 * math.pi * t)) / (2.0 * math.log(base))
        lo = max(math.floor(turns(scaling.fast)), 0)
        hi = min(math.ceil(turns(scaling.slow)), dims - 1)
        ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        freq = freq / scaling.factor * ramp + freq * (1.0 - ramp)
        magnitude = 0.1 * math.log(scaling.factor) + 1.0
    angle = torch.arange(max_position, dtype=torch.float64)[:, None] * freq[None, :]
    return torch.cat([angle.cos() * magnitude, angle.sin() * magnitude], dim=-1).float().to(device).contiguous()


# ---------------------------------------------------------------------------------------
# latent cache
# ---------------------------------------------------------------------------------------
class LatentKVCache:
    """One row per token: normed latent | rotated key part, each zero padded to the kernels' widths.  Slots are
    addressed exactly as in layers.KVCache (block table of first-slot ids)."""

    def __init__(self, n_blocks: int, block_size: int, c_pad: int, r_pad: int, dtype: torch.dtype, device):
        self._block_size = block_size
        self.c_pad = c_pad
        self.rows = torch.zeros(n_blocks * block_size, c_pad + r_pad, dtype=dtype, device=device)

    def block_size(self) -> int:
        return self._block_size


@dataclass
class LatentPlan:
    """What the portions of a step need for one attention window: the slots of every visible context row, and the
    128-row query tiles (longest context first), see slm_latent_prefill_args."""
    slots: torch.Tensor   # [n_ctx] int32
    tiles: torch.Tensor   # [n_tiles, 6] int32

    @staticmethod
    def host(portions: Sequence[Portion], window: int, block_size: int):
        slots: List[np.ndarray] = []
        tiles: List[tuple] = []
        base = 0
        for p in portions:
            start = p.kv_len - p.q_len
            first = max(0, start - window + 1) if window > 0 else 0
            pos = np.arange(first, p.kv_len)
            slots.append((np.asarray(p.blocks)[pos // block_size] + pos % block_size).astype(np.int32))
            n = p.kv_len - first
            for q0 in range(0, p.q_len, _lib.LATENT_Q_TILE):
                rows = min(_lib.LATENT_Q_TILE, p.q_len - q0)
                hi = start + q0 + rows
                lo = max(first, start + q0 - window + 1) if window > 0 else first
                tiles.append((hi - lo, (p.row0 + q0, rows, base, n, first, start + q0)))
            base += n
        tiles.sort(key=lambda t: -t[0])
        return np.concatenate(slots), np.array([t for _, t in tiles], dtype=np.int32)

    @staticmethod
    def build(portions: Sequence[Portion], window: int, block_size: int, device) -> "LatentPlan":
        slots, tiles = LatentPlan.host(portions, window, block_size)
        return LatentPlan(torch.from_numpy(slots).to(device), torch.from_numpy(tiles).to(device))


# ---------------------------------------------------------------------------------------
# latent attention
# ---------------------------------------------------------------------------------------
@dataclass
class LatentAttentionArgs:
    heads: int
    dim: int            # unrotated query / key width per head
    rot_dim: int        # rotated query / key width
    vdim: int
    kv_rank: int
    scale: float
    window: int         # positions a token sees, itself included; 0 = all
    rot_base: float
    rot_scaling: Optional[YarnScaling]


def _pad_latent(rank: int) -> int:
    for w in (64, 128, 256, 512):   # widths with an MFMA kernel
        if rank <= w:
            return w
    return round_up(rank, 64)


def _pad_query(dim: int, r_pad: int) -> int:
    d = round_up(dim, 32)
    return d + 32 if d + r_pad == 224 else d   # (widths the portion kernel has: 64 .. 192 in steps of 32, 256)


def _pad_value(v: int) -> int:
    for w in (32, 64, 128):
        if v <= w:
            return w
    return round_up(v, 32)


class LatentAttention:
    """Weights of one latent-attention mixer.  `names`: checkpoint tensors
      q [heads (dim + rot_dim), width], dkv [kv_rank + rot_dim, width], dkv.norm [kv_rank], uk [heads dim, kv_rank],
      uv [heads vdim, kv_rank], g [heads, width], o [width, heads vdim].

    Single tokens: q_abs = W_uk^T q per head, attention over the cached rows, W_uv and the gate on the result.
    Portions of at least PORTION_MIN tokens (16-bit, where the kernel has the sizes): context rows gathered and
    expanded by one product, multi-head attention over them.  32-bit: every row as a single token."""

    PORTION_MIN = 16

    def __init__(self, args: LatentAttentionArgs, width: int, eps: float, w: Dict[str, torch.Tensor], cos_sin: torch.Tensor,
                 dtype: torch.dtype, device):
        a = self.args = args
        self.eps, self.cos_sin = eps, cos_sin
        self.c_pad, self.r_pad = _pad_latent(a.kv_rank), round_up(a.rot_dim, 32)
        self.q_dim, self.v_pad = _pad_query(a.dim, self.r_pad), _pad_value(a.vdim)
        self.head_w = self.q_dim + self.r_pad
        self.off_c = a.heads * self.head_w
        self.off_r = self.off_c + self.c_pad
        self.off_g = self.off_r + self.r_pad
        n = self.off_g + round_up(a.heads, 16)
        k = round_up(width, 64)
        H = a.heads

        def z(*shape):
            return torch.zeros(*shape, dtype=dtype, device=device)
        g = {name: t.to(device=device, dtype=dtype) for name, t in w.items() if name != "dkv.norm"}
        self.w_in = z(n, k)
        q = self.w_in[:self.off_c].view(H, self.head_w, k)
        src = g["q"].view(H, a.dim + a.rot_dim, width)
        q[:, :a.dim, :width] = src[:, :a.dim]
        q[:, self.q_dim:self.q_dim + a.rot_dim, :width] = src[:, a.dim:]
        self.w_in[self.off_c:self.off_c + a.kv_rank, :width] = g["dkv"][:a.kv_rank]
        self.w_in[self.off_r:self.off_r + a.rot_dim, :width] = g["dkv"][a.kv_rank:]
        self.w_in[self.off_g:self.off_g + H, :width] = g["g"]
        self.norm = w["dkv.norm"].to(device=device, dtype=torch.float32).contiguous()
        uk, uv = g["uk"].view(H, a.dim, a.kv_rank), g["uv"].view(H, a.vdim, a.kv_rank)
        self.w_abs = z(H, self.c_pad, round_up(self.q_dim, 64))   # W_uk^T: contraction over the head's query columns
        self.w_abs[:, :a.kv_rank, :a.dim] = uk.transpose(1, 2)
        self.w_uv = z(H, self.v_pad, self.c_pad)
        self.w_uv[:, :a.vdim, :a.kv_rank] = uv
        self.portions_ok = dtype == torch.bfloat16 and lk.latent_prefill_supported(self.q_dim, self.r_pad, self.v_pad)
        self.w_ukv = None
        if self.portions_ok:
            self.w_ukv = z(H, self.q_dim + self.v_pad, self.c_pad)
            self.w_ukv[:, :a.dim, :a.kv_rank] = uk
            self.w_ukv[:, self.q_dim:self.q_dim + a.vdim, :a.kv_rank] = uv
            self.w_ukv = self.w_ukv.view(-1, self.c_pad)
        self.o_k = round_up(H * self.v_pad, 64)
        self.w_o = z(round_up(width, 16), self.o_k)
        self.w_o[:width, :H * self.v_pad].view(width, H, self.v_pad)[:, :, :a.vdim] = g["o"].view(width, H, a.vdim)

    def new_cache(self, n_blocks: int, block_size: int) -> LatentKVCache:
        return LatentKVCache(n_blocks, block_size, self.c_pad, self.r_pad, self.w_in.dtype, self.w_in.device)

    def forward(self, h: torch.Tensor, positions: torch.Tensor, cache: LatentKVCache, params: InputParameters):
        """h [rows, padded width] -> what the residual stream receives (a tensor or split-K slabs)."""
        a, T = self.args, h.size(0)
        proj = lk.linear(h, self.w_in)
        portions = params.portions if self.portions_ok else ()
        n_tok = portions[0].row0 if portions else T
        q_abs = proj.new_empty(n_tok, a.heads, self.c_pad + self.r_pad)
        lk.latent_append(proj, cache.rows, q_abs, self.norm, self.cos_sin, positions, params.new_cache_slots, heads=a.heads,
                         q_dim=self.q_dim, q_rot=self.r_pad, rank=a.kv_rank, c_pad=self.c_pad, off_c=self.off_c,
                         off_r=self.off_r, eps=self.eps)
        out = proj.new_empty(T, self.o_k)
        if self.o_k != a.heads * self.v_pad:
            out[:, a.heads * self.v_pad:].zero_()
        if n_tok:
            pt = proj[:n_tok]
            lk.linear_heads(pt, self.head_w, self.w_abs, q_abs.view(n_tok, -1), self.c_pad + self.r_pad)
            lat = proj.new_empty(n_tok, a.heads, self.c_pad)
            lk.latent_attention(q_abs, cache.rows, lat, positions, params.q_cu_seq_lens, params.block_tables,
                                params.cu_block_lens, block_size=cache.block_size(), window=a.window, scale=a.scale,
                                max_kv_len=params.kv_max_seq_len)
            lk.linear_heads(lat.view(n_tok, -1), self.c_pad, self.w_uv, out[:n_tok], self.v_pad, gate=pt[:, self.off_g:])
        if portions:
            plan = params.plans.get(a.window)
            if plan is None:
                plan = params.plans[a.window] = LatentPlan.build(portions, a.window, cache.block_size(), h.device)
            ctx = lk.latent_gather(cache.rows, plan.slots)
            kv = torch.mm(ctx[:, :self.c_pad], self.w_ukv.t())
            lk.latent_prefill(proj, ctx, kv, out, plan.tiles, heads=a.heads, q_dim=self.q_dim, c_pad=self.c_pad,
                              v_pad=self.v_pad, gate_off=self.off_g, window=a.window, scale=a.scale)
        if T <= lk.STREAM_MAX_ROWS:
            return lk.linear_slabs(out, self.w_o)
        return lk.linear(out, self.w_o)


# ---------------------------------------------------------------------------------------
# feed-forward
# ---------------------------------------------------------------------------------------
class ClampedGLU:
    """W_down (g sigmoid(alpha g) (u + shift)), g = min(W_gate h, limit), u = clamp(W_up h, +-limit); without a limit, with
    alpha 1 and shift 0, the SiLU GLU."""

    def __init__(self, width: int, ff: int, limit: float, w: Dict[str, torch.Tensor], dtype: torch.dtype, device,
                 alpha: float = lk.GLU_ALPHA, shift: float = lk.GLU_SHIFT):
        self.limit, self.alpha, self.shift = float(limit), float(alpha), float(shift)
        k, f = round_up(width, 64), round_up(ff, 64)
        self.w_gate_up = torch.zeros(2 * f, k, dtype=dtype, device=device)
        self.w_gate_up[:ff, :width] = w["gate"].to(device=device, dtype=dtype)
        self.w_gate_up[f:f + ff, :width] = w["up"].to(device=device, dtype=dtype)
        self.w_down = torch.zeros(round_up(width, 16), f, dtype=dtype, device=device)
        self.w_down[:width, :ff] = w["down"].to(device=device, dtype=dtype)

    def forward(self, h: torch.Tensor):
        act = h.new_empty(h.size(0), self.w_down.size(1))
        lk.linear_glu(h, self.w_gate_up, act, self.limit, self.alpha, self.shift)
        if h.size(0) <= lk.STREAM_MAX_ROWS:
            return lk.linear_slabs(act, self.w_down)
        return lk.linear(act, self.w_down)
