"""Python face of libslm_mixers.so (include/slm_mixers.h): recurrent layers and windowed attention with a sink.

Everything runs on torch's current stream and is hipGraph-capturable.  Shapes are checked here, on the host;
there is no fallback: a missing library or a CPU tensor raises.
"""
from __future__ import annotations

import ctypes as C
from dataclasses import dataclass
from typing import Optional

import numpy as np
import torch

from . import _lib
from ._lib import mixers_check
from .kernels import reserve_workspace
from .latent_kernels import _code, _i32, _need, _p, _stream
from .layers import InputParameters, RecurrentState


def recurrent_dim_pad(dim: int) -> int:
    """Key width of a state of `dim` key channels; raises where no kernel has it."""
    n = _lib.mixers_lib().slm_recurrent_dim_pad(dim)
    _need(n > 0, f"recurrent layers: key width {dim} is beyond the kernels' 256")
    return n


@dataclass
class RecurrentSpec:
    """Sizes, constants and fp32 weights of one recurrent layer, and where its inputs are in the projection's rows."""
    mode: int            # _lib.REC_DELTA / REC_LIGHTNING
    heads: int
    qk_heads: int
    dim: int
    vdim: int
    off_q: int
    off_k: int
    off_v: int
    eps: float
    off_b: int = 0                                 # delta
    off_gate: int = 0                              # delta: gate logits in `low`
    q_scale: float = 1.0
    unit_eps: float = 0.0
    taps: int = 0
    conv_w: Optional[torch.Tensor] = None          # [taps, channels]
    neg_a: Optional[torch.Tensor] = None           # [heads]
    dt_bias: Optional[torch.Tensor] = None         # [heads, dim]
    norm_weight: Optional[torch.Tensor] = None     # [vdim]
    decay: Optional[torch.Tensor] = None           # lightning: [heads]

    @property
    def dim_pad(self) -> int:
        return recurrent_dim_pad(self.dim)

    @property
    def v_pad(self) -> int:
        return (self.vdim + 15) // 16 * 16

    @property
    def channels(self) -> int:
        return 2 * self.qk_heads * self.dim + self.heads * self.vdim


def _f32(t: torch.Tensor, shape, what: str) -> None:
    _need(t.dtype == torch.float32 and t.is_contiguous() and tuple(t.shape) == tuple(shape), f"{what}: contiguous fp32 {list(shape)}")


def _recurrent_args(s: RecurrentSpec, proj, low, state: RecurrentState, positions, q_cu, state_slots, n_single: int):
    a = _lib.RecurrentArgs()
    T, batch = proj.size(0), q_cu.numel() - 1
    delta = s.mode == _lib.REC_DELTA
    _need(proj.dim() == 2 and proj.stride(1) == 1, "recurrent: projection rows")
    last = max(s.off_q + s.qk_heads * s.dim, s.off_k + s.qk_heads * s.dim, s.off_v + s.heads * s.vdim, s.off_b + s.heads if delta else 0)
    _need(last <= proj.size(1), "recurrent: inputs exceed the projection's rows")
    _need(s.v_pad <= 256, f"recurrent layers: value width {s.vdim} is beyond the kernels' 256")
    _i32(positions, T, "positions")
    _i32(q_cu, 2, "q_cu")
    _i32(state_slots, batch, "state_slots")
    _f32(state.state, (state.state.size(0), s.heads, s.dim_pad, s.v_pad), "recurrent state")
    _need(0 <= n_single <= batch and n_single <= T and (n_single == batch) == (n_single == T), "recurrent: single rows")
    a.proj, a.state, a.positions, a.q_cu, a.state_slots = _p(proj), _p(state.state), _p(positions), _p(q_cu), _p(state_slots)
    a.rows, a.ld_proj, a.off_q, a.off_k, a.off_v, a.off_b = T, proj.stride(0), s.off_q, s.off_k, s.off_v, s.off_b
    a.mode, a.dtype, a.batch, a.n_single, a.n_slots = s.mode, _code(proj), batch, n_single, state.state.size(0)
    a.heads, a.qk_heads, a.dim, a.vdim, a.dim_pad, a.v_pad, a.taps = s.heads, s.qk_heads, s.dim, s.vdim, s.dim_pad, s.v_pad, s.taps
    a.q_scale, a.eps, a.unit_eps = s.q_scale, s.eps, s.unit_eps
    if delta:
        _need(low.size(0) == T and low.stride(1) == 1 and low.dtype == proj.dtype and
              low.size(1) >= max(s.heads * s.dim, s.off_gate + s.heads * s.vdim), "recurrent: low-rank inputs")
        _f32(s.conv_w, (s.taps, s.channels), "convolution")
        _f32(s.neg_a, (s.heads,), "neg_a")
        _f32(s.dt_bias, (s.heads, s.dim), "dt_bias")
        _f32(s.norm_weight, (s.vdim,), "norm")
        _need(state.ring is not None and state.ring.is_contiguous() and state.ring.dtype == proj.dtype and
              tuple(state.ring.shape) == (state.state.size(0), s.taps, s.channels), "recurrent: convolution ring")
        a.low, a.ld_low, a.off_gate, a.conv_w, a.conv_ring = _p(low), low.stride(0), s.off_gate, _p(s.conv_w), _p(state.ring)
        a.neg_a, a.dt_bias, a.norm_weight = _p(s.neg_a), _p(s.dt_bias), _p(s.norm_weight)
    else:
        _f32(s.decay, (s.heads,), "decay")
        a.decay = _p(s.decay)
    return a


def recurrent_step(s: RecurrentSpec, proj: torch.Tensor, low: Optional[torch.Tensor], state: RecurrentState, positions: torch.Tensor,
                   q_cu: torch.Tensor, state_slots: torch.Tensor, n_single: int, out: Optional[torch.Tensor] = None):
    """The first n_single sequences, one row each.  Delta: normed and gated into out [n_single, >= heads vdim], zero padded.
    Lightning: read-outs [n_single, heads, v_pad] fp32 are returned, for gated_norm()."""
    a = _recurrent_args(s, proj, low, state, positions, q_cu, state_slots, n_single)
    o = None
    if s.mode == _lib.REC_DELTA:
        _need(out is not None and out.size(0) == n_single and out.stride(1) == 1 and out.dtype == proj.dtype and
              out.size(1) >= s.heads * s.vdim, "recurrent_step: out")
        # (the kernel pads up to a row's end: rows are whole)
        _need(n_single == 0 or out.stride(0) == out.size(1), "recurrent_step: out rows are contiguous")
        a.out, a.ld_out = _p(out), out.stride(0)
    else:
        o = torch.empty(n_single, s.heads, s.v_pad, dtype=torch.float32, device=proj.device)
        a.o = _p(o)
    if n_single:
        mixers_check(_lib.mixers_lib().slm_recurrent_step(C.byref(a), _stream()), "slm_recurrent_step")
    return o


@dataclass
class ChunkPlan:
    """The portions of a step in chunks of at most 16 tokens (see slm_recurrent_args)."""
    CHUNK = 16
    chunks: torch.Tensor       # [n_chunks, 3] int32: sequence, first row, rows
    seq_chunks: torch.Tensor   # [portions] int32: first chunk

    @staticmethod
    def host(portions, n_single: int):
        chunks, first = [], []
        for i, p in enumerate(portions):
            first.append(len(chunks))
            chunks += [(n_single + i, p.row0 + t, min(ChunkPlan.CHUNK, p.q_len - t)) for t in range(0, p.q_len, ChunkPlan.CHUNK)]
        return np.array(chunks, dtype=np.int32), np.array(first, dtype=np.int32)

    @staticmethod
    def of(params: InputParameters, n_single: int, device) -> "ChunkPlan":
        plan = params.plans.get("chunks")
        if plan is None:
            chunks, first = ChunkPlan.host(params.portions, n_single)
            plan = params.plans["chunks"] = ChunkPlan(torch.from_numpy(chunks).to(device), torch.from_numpy(first).to(device))
        return plan


def recurrent_portions(s: RecurrentSpec, proj: torch.Tensor, low: Optional[torch.Tensor], state: RecurrentState,
                       positions: torch.Tensor, q_cu: torch.Tensor, state_slots: torch.Tensor, n_single: int, plan: ChunkPlan) -> torch.Tensor:
    """The sequences behind the first n_single, chunk after chunk: read-outs [portion rows, heads, v_pad] fp32."""
    a = _recurrent_args(s, proj, low, state, positions, q_cu, state_slots, n_single)
    n, n_chunks, dev = proj.size(0) - n_single, plan.chunks.size(0), proj.device
    L = _lib.mixers_lib()
    o = torch.empty(n, s.heads, s.v_pad, dtype=torch.float32, device=dev)
    pre = torch.empty(n_chunks, s.heads, L.slm_recurrent_record_floats(s.dim_pad, s.v_pad), dtype=torch.float32, device=dev)
    _need(plan.chunks.dim() == 2 and plan.chunks.size(1) == 3 and n_chunks * ChunkPlan.CHUNK >= n, "recurrent: chunks")
    _i32(plan.chunks, 3 * n_chunks, "chunks")
    _i32(plan.seq_chunks, q_cu.numel() - 1 - n_single, "seq_chunks")
    a.chunks, a.seq_chunks, a.n_chunks, a.pre, a.o = _p(plan.chunks), _p(plan.seq_chunks), n_chunks, _p(pre), _p(o)
    if n:
        mixers_check(L.slm_recurrent_prepare(C.byref(a), _stream()), "slm_recurrent_prepare")
        mixers_check(L.slm_recurrent_scan(C.byref(a), _stream()), "slm_recurrent_scan")
    return o


def gated_norm(o: torch.Tensor, vdim: int, gate: torch.Tensor, weight: torch.Tensor, out: torch.Tensor, *, eps: float,
               per_head: bool, scale: float = 1.0) -> None:
    """out [rows, >= heads vdim] = scale * rms_norm(o [rows, heads, v_pad]) * weight * sigmoid(gate), zero padded; the norm is
    over a head (weight [vdim]) or over all heads (weight [heads vdim])."""
    rows, heads, v_pad = o.shape
    _f32(o, o.shape, "gated_norm: o")
    _f32(weight, (vdim if per_head else heads * vdim,), "gated_norm: weight")
    _need(gate.size(0) == rows and gate.size(1) >= heads * vdim and gate.stride(1) == 1 and gate.dtype == out.dtype, "gated_norm: gate")
    _need(out.size(0) == rows and out.size(1) >= heads * vdim and out.stride(1) == 1 and v_pad >= vdim, "gated_norm: out")
    a = _lib.GatedNormArgs()
    a.o, a.gate, a.weight, a.out = _p(o), _p(gate), _p(weight), _p(out)
    a.rows, a.ld_gate, a.ld_out, a.out_width = rows, gate.stride(0), out.stride(0), out.size(1)
    a.heads, a.vdim, a.v_pad, a.per_head, a.dtype, a.eps, a.scale = heads, vdim, v_pad, int(per_head), _code(out), float(eps), float(scale)
    if rows:
        mixers_check(_lib.mixers_lib().slm_gated_norm(C.byref(a), _stream()), "slm_gated_norm")


def window_append(proj: torch.Tensor, key_cache: torch.Tensor, value_cache: torch.Tensor, q_weight: torch.Tensor,
                  k_weight: torch.Tensor, cos_sin: torch.Tensor, positions: torch.Tensor, slots: torch.Tensor, *, heads: int, dim: int,
                  off_q: int, off_k: int, off_v: int, eps: float) -> None:
    """Norm per head and rotation: queries in place, keys (and values) into the cache."""
    rows = proj.size(0)
    G, d_pad, v_pad = key_cache.size(1), key_cache.size(2), value_cache.size(2)
    _need(proj.stride(1) == 1 and key_cache.is_contiguous() and value_cache.is_contiguous() and
          proj.dtype == key_cache.dtype == value_cache.dtype and value_cache.shape[:2] == key_cache.shape[:2], "window_append: cache")
    _need(max(off_q + heads * d_pad, off_k + G * d_pad, off_v + G * v_pad) <= proj.size(1), "window_append: projection rows")
    _f32(q_weight, (dim,), "q norm")
    _f32(k_weight, (dim,), "k norm")
    _need(cos_sin.dtype == torch.float32 and cos_sin.is_contiguous() and cos_sin.dim() == 2, "window_append: cos_sin")
    _i32(positions, rows, "positions")
    _i32(slots, rows, "slots")
    a = _lib.WindowAppendArgs()
    a.proj, a.key_cache, a.value_cache, a.q_weight, a.k_weight = _p(proj), _p(key_cache), _p(value_cache), _p(q_weight), _p(k_weight)
    a.cos_sin, a.positions, a.slots = _p(cos_sin), _p(positions), _p(slots)
    a.rows, a.ld_proj, a.off_q, a.off_k, a.off_v = rows, proj.stride(0), off_q, off_k, off_v
    a.max_positions, a.n_slots = cos_sin.size(0), key_cache.size(0)
    a.heads, a.kv_heads, a.dim, a.rot, a.d_pad, a.v_pad, a.dtype, a.eps = heads, G, dim, cos_sin.size(1), d_pad, v_pad, _code(proj), float(eps)
    mixers_check(_lib.mixers_lib().slm_window_append(C.byref(a), _stream()), "slm_window_append")


def window_attention(q: torch.Tensor, key_cache: torch.Tensor, value_cache: torch.Tensor, out: torch.Tensor,
                     sink: Optional[torch.Tensor], positions: torch.Tensor, q_cu: torch.Tensor, block_table: torch.Tensor,
                     block_cu: torch.Tensor, *, heads: int, block_size: int, window: int, keep_first: int, scale: float, softcap: float,
                     max_kv_len: int, out_scale: float = 1.0, n_splits: int = 0, generic: bool = False) -> None:
    """Every row on its own: q [rows, >= heads d_pad] -> out [rows, >= heads v_pad]."""
    rows = q.size(0)
    G, d_pad, v_pad = key_cache.size(1), key_cache.size(2), value_cache.size(2)
    _need(q.stride(1) == 1 and out.stride(1) == 1 and q.size(1) >= heads * d_pad and out.size(1) >= heads * v_pad and
          out.size(0) == rows and q.dtype == key_cache.dtype == value_cache.dtype == out.dtype and key_cache.is_contiguous() and
          value_cache.is_contiguous(), "window_attention: shapes")
    if sink is not None:
        _f32(sink, (heads,), "sink")
    n = q_cu.numel() - 1
    _i32(positions, rows, "positions")
    _i32(q_cu, 2, "q_cu")
    _i32(block_cu, n + 1, "block_cu")
    _i32(block_table, 1, "block_table")
    a = _lib.WindowAttnArgs()
    a.q, a.key_cache, a.value_cache, a.out, a.sink = _p(q), _p(key_cache), _p(value_cache), _p(out), _p(sink)
    a.positions, a.q_cu, a.block_table, a.block_cu = _p(positions), _p(q_cu), _p(block_table), _p(block_cu)
    a.rows, a.ld_q, a.ld_out, a.batch, a.heads, a.kv_heads, a.d_pad, a.v_pad = rows, q.stride(0), out.stride(0), n, heads, G, d_pad, v_pad
    a.block_size, a.window, a.keep_first, a.max_kv_len, a.n_splits = block_size, window, keep_first, max_kv_len, n_splits
    a.scale, a.softcap, a.out_scale, a.dtype, a.generic = float(scale), float(softcap), float(out_scale), _code(q), int(generic)
    L = _lib.mixers_lib()
    need = L.slm_window_attn_workspace_bytes(C.byref(a))
    if need:
        ws = reserve_workspace(need, q.device)
        a.workspace, a.workspace_bytes = ws.data_ptr(), ws.numel()
    mixers_check(L.slm_window_attn(C.byref(a), _stream()), "slm_window_attn")


def window_prefill_supported(d_pad: int, v_pad: int) -> bool:
    return bool(_lib.mixers_lib().slm_window_prefill_supported(d_pad, v_pad))


def window_prefill(q: torch.Tensor, key_cache: torch.Tensor, value_cache: torch.Tensor, out: torch.Tensor, sink: Optional[torch.Tensor],
                   slots: torch.Tensor, tiles: torch.Tensor, *, heads: int, window: int, keep_first: int, scale: float, softcap: float,
                   out_scale: float = 1.0) -> None:
    """The portions' rows over their context (mixer_layers.WindowPlan)."""
    G, d_pad, v_pad = key_cache.size(1), key_cache.size(2), value_cache.size(2)
    _need(q.dtype == key_cache.dtype == value_cache.dtype == out.dtype == torch.bfloat16, "window_prefill: bfloat16")
    _need(q.stride(1) == 1 and out.stride(1) == 1 and q.size(1) >= heads * d_pad and out.size(1) >= heads * v_pad and
          q.size(0) == out.size(0) and key_cache.is_contiguous() and value_cache.is_contiguous(), "window_prefill: shapes")
    _need(tiles.dim() == 2 and tiles.size(1) == 7, "window_prefill: tiles")
    _i32(tiles, tiles.numel(), "tiles")
    _i32(slots, 1, "slots")
    if sink is not None:
        _f32(sink, (heads,), "sink")
    a = _lib.WindowPrefillArgs()
    a.q, a.key_cache, a.value_cache, a.out, a.sink = _p(q), _p(key_cache), _p(value_cache), _p(out), _p(sink)
    a.slots, a.tiles, a.ld_q, a.ld_out, a.n_rows, a.n_ctx = _p(slots), _p(tiles), q.stride(0), out.stride(0), q.size(0), slots.numel()
    a.n_tiles, a.heads, a.kv_heads, a.d_pad, a.v_pad, a.window, a.keep_first = tiles.size(0), heads, G, d_pad, v_pad, window, keep_first
    a.scale, a.softcap, a.out_scale = float(scale), float(softcap), float(out_scale)
    mixers_check(_lib.mixers_lib().slm_window_prefill(C.byref(a), _stream()), "slm_window_prefill")
