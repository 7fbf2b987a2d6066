"""Token mixers over libslm_mixers: windowed grouped-query attention with kept first tokens, capped scores and a sink;
decayed linear ("lightning") attention; the gated delta rule with a decay per key channel; and two mixers side by side.

A mixer's projections of its input are one product (w_in) and its heads enter one output product (w_o).  Rows of a step
are single tokens first, then portions (InputParameters.portions): each has its own kernels.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Dict, List, Optional, Sequence

import numpy as np
import torch

from . import _lib
from . import latent_kernels as lk
from . import mixer_kernels as mk
from .kernels import SlmError
from .latent_layers import round_up
from .layers import InputParameters, KVCache, Portion, RecurrentState


def single_rows(params: InputParameters, rows: int) -> int:
    """Rows in front of the portions: one per sequence."""
    if params.portions:
        return params.portions[0].row0
    if rows != params.q_cu_seq_lens.numel() - 1:
        raise SlmError("sequences that bring several tokens are described as portions")
    return rows


def out_product(x: torch.Tensor, w: torch.Tensor):
    """What the residual stream receives: split-K slabs for few rows, a tensor otherwise."""
    return lk.linear_slabs(x, w) if x.size(0) <= lk.STREAM_MAX_ROWS else lk.linear(x, w)


def _rows_of(n: int, k: int, width: int, parts, dtype, device) -> torch.Tensor:
    """[n, k] of zeros with `parts` (first row, weight [rows, width]) laid in."""
    w = torch.zeros(n, k, dtype=dtype, device=device)
    for at, t in parts:
        w[at:at + t.size(0), :width] = t.to(device=device, dtype=dtype)
    return w


# ---------------------------------------------------------------------------------------
# windowed attention
# ---------------------------------------------------------------------------------------
@dataclass
class WindowAttentionArgs:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot_base: float
    rot_dims: int
    softcap: float = 0.0     # 0 = none
    window: int = 0          # positions a token sees, itself included; 0 = all
    keep_first: int = 0      # first positions that stay visible


@dataclass
class WindowPlan:
    """What the portions of a step need for one (window, kept tokens): cache slots of every context row, and the query
    tiles (most keys first), see slm_window_prefill_args."""
    slots: torch.Tensor   # [n_ctx] int32
    tiles: torch.Tensor   # [n_tiles, 7] int32

    @staticmethod
    def host(portions: Sequence[Portion], window: int, keep_first: int, block_size: int):
        slots: List[np.ndarray] = []
        tiles: List[tuple] = []
        base = 0
        for p in portions:
            start = p.kv_len - p.q_len
            first = max(0, start - window + 1) if window > 0 else 0
            kept = min(keep_first, first)
            pos = np.concatenate([np.arange(kept), np.arange(first, p.kv_len)])
            slots.append((np.asarray(p.blocks)[pos // block_size] + pos % block_size).astype(np.int32))
            for q0 in range(0, p.q_len, _lib.WINDOW_Q_TILE):
                rows = min(_lib.WINDOW_Q_TILE, p.q_len - q0)
                last = start + q0 + rows
                keys = min(last, window + rows + keep_first) if window > 0 else last
                tiles.append((keys, (p.row0 + q0, rows, base, pos.size, kept, first, start + q0)))
            base += pos.size
        tiles.sort(key=lambda t: -t[0])
        return np.concatenate(slots), np.array([t for _, t in tiles], dtype=np.int32)

    @staticmethod
    def of(params: InputParameters, window: int, keep_first: int, block_size: int, device) -> "WindowPlan":
        key = ("window", window, keep_first)
        plan = params.plans.get(key)
        if plan is None:
            slots, tiles = WindowPlan.host(params.portions, window, keep_first, block_size)
            plan = params.plans[key] = WindowPlan(torch.from_numpy(slots).to(device), torch.from_numpy(tiles).to(device))
        return plan


def _pad_head(d: int) -> int:
    for w in (64, 96, 128, 192, 256):   # widths with MFMA kernels
        if d <= w:
            return w
    return round_up(d, 32)


class WindowAttention:
    """`w`: q [heads dim, width], k [kv_heads dim, width], v [kv_heads vdim, width], q.norm, k.norm [dim], sink [heads],
    o [width, heads vdim].  out_scale multiplies the heads' outputs."""

    def __init__(self, args: WindowAttentionArgs, width: int, eps: float, w: Dict[str, torch.Tensor], cos_sin: torch.Tensor,
                 dtype: torch.dtype, device, out_scale: float = 1.0):
        a = self.args = args
        self.eps, self.cos_sin, self.out_scale, self.dtype, self.device = eps, cos_sin, out_scale, dtype, device
        if a.heads % a.kv_heads:
            raise SlmError(f"{a.heads} query heads over {a.kv_heads} key heads")
        H, G, D, V = a.heads, a.kv_heads, a.dim, a.vdim
        self.d_pad, self.v_pad = _pad_head(D), _pad_head(V)
        self.off_k = H * self.d_pad
        self.off_v = self.off_k + G * self.d_pad
        k = round_up(width, 64)
        self.w_in = torch.zeros(self.off_v + G * self.v_pad, k, dtype=dtype, device=device)
        for at, n, d, pad, name in ((0, H, D, self.d_pad, "q"), (self.off_k, G, D, self.d_pad, "k"), (self.off_v, G, V, self.v_pad, "v")):
            self.w_in[at:at + n * pad].view(n, pad, k)[:, :d, :width] = w[name].to(device=device, dtype=dtype).view(n, d, width)
        self.out_width = H * self.v_pad
        self.w_o = torch.zeros(width, self.out_width, dtype=dtype, device=device)
        self.w_o.view(width, H, self.v_pad)[:, :, :V] = w["o"].to(device=device, dtype=dtype).view(width, H, V)
        f32 = lambda t: t.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
        self.q_norm, self.k_norm, self.sink = f32(w["q.norm"]), f32(w["k.norm"]), f32(w["sink"])
        self.prefill_ok = dtype == torch.bfloat16 and mk.window_prefill_supported(self.d_pad, self.v_pad)

    def new_cache(self, limits) -> KVCache:
        return KVCache(limits.n_blocks, limits.block_size, self.args.kv_heads, self.d_pad, self.dtype, self.device, self.v_pad)

    def forward(self, proj: torch.Tensor, positions: torch.Tensor, cache: KVCache, params: InputParameters, out: torch.Tensor) -> None:
        """proj: the rows' projections (overwritten); out [rows, out_width]."""
        a = self.args
        keys, values = cache.get_kv_cache()
        mk.window_append(proj, keys, values, self.q_norm, self.k_norm, self.cos_sin, positions, params.new_cache_slots, heads=a.heads,
                         dim=a.dim, off_q=0, off_k=self.off_k, off_v=self.off_v, eps=self.eps)
        common = dict(heads=a.heads, window=a.window, keep_first=a.keep_first, scale=a.scale, softcap=a.softcap, out_scale=self.out_scale)
        portions = params.portions if self.prefill_ok else ()
        n = portions[0].row0 if portions else proj.size(0)
        if n:
            mk.window_attention(proj[:n], keys, values, out[:n], self.sink, positions, params.q_cu_seq_lens, params.block_tables,
                                params.cu_block_lens, block_size=cache.block_size(), max_kv_len=params.kv_max_seq_len, **common)
        if portions:
            plan = WindowPlan.of(params, a.window, a.keep_first, cache.block_size(), proj.device)
            mk.window_prefill(proj, keys, values, out, self.sink, plan.slots, plan.tiles, **common)


# ---------------------------------------------------------------------------------------
# lightning attention
# ---------------------------------------------------------------------------------------
@dataclass
class LightningArgs:
    heads: int
    dim: int
    vdim: int
    decay: Sequence[float]   # per head


class LightningAttention:
    """`w`: q, k [heads dim, width], v, g [heads vdim, width], norm [heads vdim], o [width, heads vdim].  silu(q), silu(k),
    silu(v); S <- decay S + k v^T; S^T q normed over all heads and gated.  out_scale multiplies the result."""

    def __init__(self, args: LightningArgs, width: int, eps: float, w: Dict[str, torch.Tensor], dtype: torch.dtype, device,
                 out_scale: float = 1.0):
        a = self.args = args
        self.eps, self.out_scale, self.device = eps, out_scale, device
        if len(a.decay) != a.heads:
            raise SlmError(f"{len(a.decay)} decays for {a.heads} heads")
        qk, vo = a.heads * a.dim, a.heads * a.vdim
        self.off_g = 2 * qk + vo
        self.w_in = _rows_of(round_up(self.off_g + vo, 16), round_up(width, 64), width,
                             [(0, w["q"]), (qk, w["k"]), (2 * qk, w["v"]), (self.off_g, w["g"])], dtype, device)
        self.out_width = vo
        self.w_o = w["o"].to(device=device, dtype=dtype)
        self.norm = w["norm"].to(device=device, dtype=torch.float32).contiguous()
        self.spec = mk.RecurrentSpec(_lib.REC_LIGHTNING, a.heads, a.heads, a.dim, a.vdim, 0, qk, 2 * qk, eps,
                                     decay=torch.tensor(list(a.decay), dtype=torch.float32, device=device))

    def new_state(self, limits) -> RecurrentState:
        a = self.args
        return RecurrentState(limits.n_states, a.heads, self.spec.dim_pad, self.spec.v_pad, self.device)

    def forward(self, proj: torch.Tensor, positions: torch.Tensor, state: RecurrentState, params: InputParameters, out: torch.Tensor) -> None:
        """proj: the rows' projections; out [rows, >= out_width], zero padded."""
        n = single_rows(params, proj.size(0))
        step = (self.spec, proj, None, state, positions, params.q_cu_seq_lens, params.state_slots, n)
        gate = proj[:, self.off_g:]
        how = dict(eps=self.eps, per_head=False, scale=self.out_scale)
        if n:
            mk.gated_norm(mk.recurrent_step(*step), self.args.vdim, gate[:n], self.norm, out[:n], **how)
        if n < proj.size(0):
            mk.gated_norm(mk.recurrent_portions(*step, mk.ChunkPlan.of(params, n, proj.device)), self.args.vdim, gate[n:], self.norm, out[n:], **how)


# ---------------------------------------------------------------------------------------
# two mixers side by side
# ---------------------------------------------------------------------------------------
class ParallelMixer:
    """Windowed attention and lightning attention on the same input: one product in front, one behind (the mixers' scales
    are applied to the heads' outputs)."""

    def __init__(self, left: WindowAttention, right: LightningAttention, width: int):
        self.left, self.right = left, right
        self.split = left.w_in.size(0)
        self.w_in = torch.cat([left.w_in, right.w_in])
        self.o_k = round_up(left.out_width + right.out_width, 64)
        self.w_o = torch.zeros(round_up(width, 16), self.o_k, dtype=left.dtype, device=self.w_in.device)
        self.w_o[:width, :left.out_width] = left.w_o
        self.w_o[:width, left.out_width:left.out_width + right.out_width] = right.w_o
        left.w_in = right.w_in = left.w_o = right.w_o = None   # (laid out once)

    def new_cache(self, limits):
        return self.left.new_cache(limits), self.right.new_state(limits)

    def forward(self, h: torch.Tensor, positions: torch.Tensor, cache, params: InputParameters):
        proj = lk.linear(h, self.w_in)
        out = proj.new_empty(h.size(0), self.o_k)
        self.left.forward(proj[:, :self.split], positions, cache[0], params, out[:, :self.left.out_width])
        self.right.forward(proj[:, self.split:], positions, cache[1], params, out[:, self.left.out_width:])
        return out_product(out, self.w_o)


# ---------------------------------------------------------------------------------------
# gated delta rule
# ---------------------------------------------------------------------------------------
@dataclass
class ChannelDeltaArgs:
    heads: int
    kv_heads: int    # q / k heads
    dim: int
    vdim: int
    taps: int


class ChannelDelta:
    """`w`: q, k [kv_heads dim, width], v [heads vdim, width], their .conv [channels, taps], b [heads, width], A_log [heads],
    a1 [r, width], a2 [heads dim, r], dt_bias [heads dim], g1 [r', width], g2 [heads vdim, r'], norm [vdim],
    o [width, heads vdim]."""

    UNIT_EPS = 1e-6

    def __init__(self, args: ChannelDeltaArgs, width: int, eps: float, w: Dict[str, torch.Tensor], dtype: torch.dtype, device):
        a = self.args = args
        self.eps, self.dtype, self.device = eps, dtype, device
        H, G, D, V = a.heads, a.kv_heads, a.dim, a.vdim
        if H % G:
            raise SlmError(f"{H} heads over {G} key heads")
        qk, vo = G * D, H * V
        ra, rg = w["a1"].size(0), w["g1"].size(0)
        self.low_k = round_up(max(ra, rg, 1), 64)
        self.low_n = round_up(max(H * D, vo), 16)
        off_b = 2 * qk + vo
        self.off_a1 = round_up(off_b + H, 64)
        self.w_in = _rows_of(self.off_a1 + 2 * self.low_k, round_up(width, 64), width,
                             [(0, w["q"]), (qk, w["k"]), (2 * qk, w["v"]), (off_b, w["b"]), (self.off_a1, w["a1"]),
                              (self.off_a1 + self.low_k, w["g1"])], dtype, device)
        self.w_low = torch.zeros(2, self.low_n, self.low_k, dtype=dtype, device=device)
        self.w_low[0, :H * D, :ra] = w["a2"].to(device=device, dtype=dtype)
        self.w_low[1, :vo, :rg] = w["g2"].to(device=device, dtype=dtype)
        self.o_k = round_up(vo, 64)
        self.w_o = torch.zeros(round_up(width, 16), self.o_k, dtype=dtype, device=device)
        self.w_o[:width, :vo] = w["o"].to(device=device, dtype=dtype)
        f32 = lambda t: t.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
        self.spec = mk.RecurrentSpec(
            _lib.REC_DELTA, H, G, D, V, 0, qk, 2 * qk, eps, off_b=off_b, off_gate=self.low_n, q_scale=D ** -0.5, unit_eps=self.UNIT_EPS,
            taps=a.taps, conv_w=f32(torch.cat([w[n + ".conv"] for n in "qkv"]).t()), neg_a=f32(-torch.exp(w["A_log"].double())),
            dt_bias=f32(w["dt_bias"].view(H, D)), norm_weight=f32(w["norm"]))

    def new_cache(self, limits) -> RecurrentState:
        s = self.spec
        return RecurrentState(limits.n_states, s.heads, s.dim_pad, s.v_pad, self.device, s.taps, s.channels, self.dtype)

    def forward(self, h: torch.Tensor, positions: torch.Tensor, state: RecurrentState, params: InputParameters):
        s, T = self.spec, h.size(0)
        n = single_rows(params, T)
        proj = lk.linear(h, self.w_in)
        low_in = proj[:, self.off_a1:]
        low = proj.new_empty(T, 2 * self.low_n)
        if lk.streams_rows(h):
            lk.linear_heads(low_in, self.low_k, self.w_low, low, self.low_n)
        else:
            for i in range(2):
                lk.linear(low_in[:, i * self.low_k:(i + 1) * self.low_k], self.w_low[i], low[:, i * self.low_n:(i + 1) * self.low_n])
        out = proj.new_empty(T, self.o_k)
        step = (s, proj, low, state, positions, params.q_cu_seq_lens, params.state_slots, n)
        if n:
            mk.recurrent_step(*step, out=out[:n])
        if n < T:
            mk.gated_norm(mk.recurrent_portions(*step, mk.ChunkPlan.of(params, n, proj.device)), s.vdim, low[n:, self.low_n:], s.norm_weight, out[n:], eps=self.eps, per_head=True)
        return out_product(out, self.w_o)
