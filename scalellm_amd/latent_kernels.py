"""Python face of libslm_latent.so (include/slm_latent.h): the dense 16- / 32-bit ops and latent attention.

Everything runs on torch's current stream and is hipGraph-capturable.  Shapes are checked here, on the host;
there is no fallback: a missing library or a CPU tensor raises.
"""
from __future__ import annotations

import ctypes as C
from typing import Optional, Tuple

import torch

from . import _lib
from ._lib import SLM_BF16, SLM_F32, SlmError, latent_check
from .kernels import reserve_workspace

# rows up to which the weight-streaming kernel serves a bf16 product; above it the vendor GEMM does
STREAM_MAX_ROWS = 32
# clamped GLU: y = g * sigmoid(alpha * g) * (u + shift)
GLU_ALPHA, GLU_SHIFT = 1.702, 1.0


def _code(t: torch.Tensor) -> int:
    if t.dtype == torch.bfloat16:
        return SLM_BF16
    if t.dtype == torch.float32:
        return SLM_F32
    raise SlmError(f"unsupported dtype {t.dtype}: bfloat16 / float32 only")


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _p(t: Optional[torch.Tensor]):
    if t is None:
        return None
    if not t.is_cuda:
        raise SlmError("libslm_latent needs GPU tensors (no CPU fallback)")
    return t.data_ptr()


def _need(ok: bool, what: str) -> None:
    if not ok:
        raise SlmError(what)


def _i32(t: torch.Tensor, n: int, what: str) -> None:
    _need(t.dtype == torch.int32 and t.is_contiguous() and t.numel() >= n, f"{what}: contiguous int32 [>= {n}]")


class TanhNorm:
    """tanh(alpha x) * weight + bias in place of a norm's statistics; given to residual_norm() as its weight."""
    __slots__ = ("alpha", "weight", "bias")

    def __init__(self, alpha: float, weight: torch.Tensor, bias: torch.Tensor):
        self.alpha, self.weight, self.bias = float(alpha), weight, bias


class Slabs:
    """fp32 split-K partial sums [n, rows, ld] that residual_norm() adds up."""
    __slots__ = ("t",)

    def __init__(self, t: torch.Tensor):
        self.t = t


def residual_norm(resid: torch.Tensor, out: Optional[torch.Tensor], weight, eps: float,
                  delta=None, embed=None, row_index: Optional[torch.Tensor] = None, mult: float = 1.0) -> None:
    """resid (fp32 [rows, width]) += mult * delta (a [rows, >= width] tensor or Slabs), or
    resid = mult * (table[tokens] (+ pos[positions])) for embed = (tokens, table, positions, pos); then
    out = rms_norm(resid) * weight, or a TanhNorm given as weight, zero padded to out's width.  weight = None: the sum only.
    row_index: out row r is the norm of stream row row_index[r]; nothing is added."""
    a = _lib.ResidualNormArgs()
    rows, width = resid.shape
    _need(resid.dtype == torch.float32 and resid.is_contiguous(), "residual_norm: resid is contiguous fp32")
    ref = out if out is not None else (delta if isinstance(delta, torch.Tensor) else None)
    a.resid, a.width, a.eps, a.delta_mult = _p(resid), width, float(eps), float(mult)
    if embed is not None:
        tokens, table, positions, pos = embed
        _i32(tokens, rows, "tokens")
        _need(table.dim() == 2 and table.stride(1) == 1 and table.size(1) >= width, "residual_norm: embedding table")
        a.mode, a.tokens, a.embed, a.ld_embed = _lib.RN_EMBED, _p(tokens), _p(table), table.stride(0)
        ref = table
        if pos is not None:
            _i32(positions, rows, "positions")
            _need(pos.is_contiguous() and pos.size(1) == width and pos.dtype == table.dtype, "residual_norm: position table")
            a.positions, a.pos_table = _p(positions), _p(pos)
    elif isinstance(delta, Slabs):
        t = delta.t
        _need(t.dtype == torch.float32 and t.is_contiguous() and t.dim() == 3 and t.size(1) == rows and t.size(2) >= width,
              "residual_norm: slabs are fp32 [n, rows, >= width]")
        a.mode, a.slabs, a.n_slabs, a.ld_delta, a.slab_stride = _lib.RN_SLABS, _p(t), t.size(0), t.size(2), t.stride(0)
    elif delta is not None:
        _need(delta.size(0) == rows and delta.size(1) >= width and delta.stride(1) == 1, "residual_norm: delta [rows, >= width]")
        _need(out is None or out.dtype == delta.dtype, "residual_norm: dtypes")
        a.mode, a.delta, a.ld_delta = _lib.RN_ADD, _p(delta), delta.stride(0)
    else:
        a.mode = _lib.RN_PLAIN
        if row_index is not None:
            _need(out is not None, "residual_norm: row_index needs an output")
            rows = out.size(0)
            _i32(row_index, rows, "row_index")
            a.row_index = _p(row_index)
    a.rows = rows
    if isinstance(weight, TanhNorm):
        t, weight = weight, weight.weight
        _need(t.bias.dtype == torch.float32 and t.bias.numel() == width and t.bias.is_contiguous(), "norm bias: fp32 [width]")
        a.norm, a.norm_alpha, a.bias = _lib.NORM_TANH, t.alpha, _p(t.bias)
    if weight is not None:
        _need(weight.dtype == torch.float32 and weight.numel() == width and weight.is_contiguous(), "norm weight: fp32 [width]")
        _need(out.size(0) == rows and out.stride(1) == 1 and out.size(1) >= width, "residual_norm: out [rows, >= width]")
        a.weight, a.out, a.ld_out = _p(weight), _p(out), out.size(1)
        _need(out.stride(0) == out.size(1), "residual_norm: out rows are contiguous")
    a.dtype = _code(ref) if ref is not None else SLM_F32
    latent_check(_lib.latent_lib().slm_residual_norm(C.byref(a), _stream()), "slm_residual_norm")


def _linear_args(x, w, M, N, K) -> "_lib.LinearArgs":
    a = _lib.LinearArgs()
    a.x, a.w, a.M, a.N, a.K = _p(x), _p(w), M, N, K
    a.alpha, a.batch, a.n_splits, a.dtype = 1.0, 1, 1, _code(w)
    return a


def _run_linear(a) -> None:
    latent_check(_lib.latent_lib().slm_linear(C.byref(a), _stream()), "slm_linear")


def _check_xw(x, w) -> Tuple[int, int, int]:
    _need(x.dim() == 2 and w.dim() == 2 and x.dtype == w.dtype and x.size(1) == w.size(1) and x.stride(1) == 1 and
          w.is_contiguous(), "linear: x [M, K], w [N, K] contiguous, one dtype")
    return x.size(0), w.size(0), w.size(1)


def streams_rows(x: torch.Tensor) -> bool:
    """Does the weight-streaming kernel serve this row count (32-bit: always)?"""
    return x.dtype == torch.float32 or x.size(0) <= STREAM_MAX_ROWS


def linear(x: torch.Tensor, w: torch.Tensor, out: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x [M, K] W[N, K]^T -> [M, N] of the same dtype."""
    M, N, K = _check_xw(x, w)
    if out is None:
        out = torch.empty(M, N, dtype=x.dtype, device=x.device)
    _need(out.shape == (M, N) and out.stride(1) == 1 and out.dtype == x.dtype, "linear: out [M, N]")
    if not streams_rows(x):
        return torch.mm(x, w.t(), out=out)
    a = _linear_args(x, w, M, N, K)
    a.ldx, a.ldw, a.ldy, a.y, a.epilogue = x.stride(0), K, out.stride(0), _p(out), _lib.LIN_STORE
    _run_linear(a)
    return out


def linear_f32(x: torch.Tensor, w: torch.Tensor, alpha: float = 1.0) -> torch.Tensor:
    """alpha * x W^T as fp32 (logits)."""
    M, N, K = _check_xw(x, w)
    out = torch.empty(M, N, dtype=torch.float32, device=x.device)
    a = _linear_args(x, w, M, N, K)
    a.ldx, a.ldw, a.ldy, a.y, a.epilogue, a.alpha = x.stride(0), K, N, _p(out), _lib.LIN_F32, float(alpha)
    _run_linear(a)
    return out


def split_count(rows: int, n_out: int, k: int) -> int:
    """Split-K slabs of a narrow product: enough workgroups for the chip, at least 4 steps of 64 per wave."""
    per = 16 if rows <= 16 else 32
    wgs = (n_out + per - 1) // per
    return max(1, min(8, 768 // max(wgs, 1), k // 1024))


def linear_slabs(x: torch.Tensor, w: torch.Tensor) -> Slabs:
    """x W^T left as fp32 split-K partial sums for residual_norm()."""
    M, N, K = _check_xw(x, w)
    n = split_count(M, N, K)
    out = torch.empty(n, M, N, dtype=torch.float32, device=x.device)
    a = _linear_args(x, w, M, N, K)
    a.ldx, a.ldw, a.ldy, a.y, a.epilogue, a.n_splits = x.stride(0), K, N, _p(out), _lib.LIN_SLABS, n
    _run_linear(a)
    return Slabs(out)


def linear_glu(x: torch.Tensor, w_gate_up: torch.Tensor, out: torch.Tensor, limit: float, alpha: float = GLU_ALPHA,
               shift: float = GLU_SHIFT) -> torch.Tensor:
    """out = clamped GLU of the two halves of x [gate | up]^T: the activation is the product's epilogue where the
    streaming kernel runs, one more launch behind the vendor GEMM otherwise."""
    M, N, K = _check_xw(x, w_gate_up)
    half = N // 2
    _need(out.shape == (M, half) and out.stride(1) == 1 and out.dtype == x.dtype, "linear_glu: out [M, N / 2]")
    if streams_rows(x):
        a = _linear_args(x, w_gate_up, M, N, K)
        a.ldx, a.ldw, a.ldy, a.y, a.epilogue = x.stride(0), K, out.stride(0), _p(out), _lib.LIN_GLU
        a.limit, a.glu_alpha, a.glu_shift = float(limit), float(alpha), float(shift)
        _run_linear(a)
    else:
        gu = torch.mm(x, w_gate_up.t())
        clamped_glu(gu, out, limit, alpha, shift)
    return out


def clamped_glu(gate_up: torch.Tensor, out: torch.Tensor, limit: float, alpha: float = GLU_ALPHA,
                shift: float = GLU_SHIFT) -> None:
    M, N = gate_up.shape
    _need(out.shape == (M, N // 2) and gate_up.stride(1) == 1 and out.stride(1) == 1 and gate_up.dtype == out.dtype,
          "clamped_glu: gate_up [M, 2 n], out [M, n]")
    latent_check(_lib.latent_lib().slm_clamped_glu(_p(out), _p(gate_up), M, N // 2, gate_up.stride(0), out.stride(0), float(limit),
                                                   float(alpha), float(shift), _code(out), _stream()), "slm_clamped_glu")


def linear_heads(x: torch.Tensor, x_head: int, w: torch.Tensor, out: torch.Tensor, out_head: int,
                 gate: Optional[torch.Tensor] = None) -> None:
    """Per-head products: head h of `out` (columns from h * out_head) = columns from h * x_head of x times w[h]^T;
    w [heads, N, K].  gate [rows, >= heads]: the result is multiplied by sigmoid(gate[:, h])."""
    H, N, K = w.shape
    M = x.size(0)
    _need(x.dim() == 2 and out.dim() == 2 and out.size(0) == M and w.is_contiguous() and x.dtype == w.dtype == out.dtype and
          x.stride(1) == 1 and out.stride(1) == 1, "linear_heads: x [M, ..], w [heads, N, K], out [M, ..]")
    _need((H - 1) * x_head + K <= x.size(1) and (H - 1) * out_head + N <= out.size(1), "linear_heads: heads exceed the rows")
    a = _linear_args(x, w, M, N, K)
    a.ldx, a.ldw, a.ldy, a.y = x.stride(0), K, out.stride(0), _p(out)
    a.batch, a.x_batch, a.w_batch, a.y_batch = H, x_head, N * K, out_head
    a.epilogue = _lib.LIN_STORE
    if gate is not None:
        _need(gate.size(0) == M and gate.size(1) >= H and gate.stride(1) == 1 and gate.dtype == x.dtype, "linear_heads: gate")
        a.epilogue, a.gate, a.ld_gate = _lib.LIN_GATE, _p(gate), gate.stride(0)
    _run_linear(a)


def latent_append(proj: torch.Tensor, cache: torch.Tensor, q_abs: Optional[torch.Tensor], norm_weight: torch.Tensor,
                  cos_sin: torch.Tensor, positions: torch.Tensor, slots: torch.Tensor, *, heads: int, q_dim: int, q_rot: int,
                  rank: int, c_pad: int, off_c: int, off_r: int, eps: float) -> None:
    """Latent RMS norm + rotation -> cache rows; the queries' rotated part in place (and behind c_pad of q_abs)."""
    rows = proj.size(0)
    a = _lib.LatentAppendArgs()
    _need(proj.stride(1) == 1 and cache.dim() == 2 and cache.is_contiguous() and cache.dtype == proj.dtype, "latent_append: cache")
    _need(cos_sin.dtype == torch.float32 and cos_sin.is_contiguous() and norm_weight.dtype == torch.float32 and
          norm_weight.numel() == rank, "latent_append: fp32 tables")
    _i32(positions, rows, "positions")
    _i32(slots, rows, "slots")
    a.proj, a.cache, a.norm_weight, a.cos_sin = _p(proj), _p(cache), _p(norm_weight), _p(cos_sin)
    a.positions, a.slots, a.rows, a.ld_proj = _p(positions), _p(slots), rows, proj.stride(0)
    a.off_c, a.off_r, a.max_positions = off_c, off_r, cos_sin.size(0)
    a.heads, a.q_dim, a.q_rot, a.rank, a.rot = heads, q_dim, q_rot, rank, cos_sin.size(1)
    a.c_pad, a.r_pad, a.dtype, a.eps = c_pad, cache.size(1) - c_pad, _code(proj), float(eps)
    if q_abs is not None and q_abs.size(0):
        _need(q_abs.is_contiguous() and q_abs.shape[1:] == (heads, cache.size(1)) and q_abs.size(0) <= rows, "latent_append: q_abs")
        a.q_abs, a.abs_rows = _p(q_abs), q_abs.size(0)
    latent_check(_lib.latent_lib().slm_latent_append(C.byref(a), _stream()), "slm_latent_append")


def latent_attention(q_abs: torch.Tensor, cache: torch.Tensor, out: torch.Tensor, positions: torch.Tensor, q_cu: torch.Tensor,
                     block_table: torch.Tensor, block_cu: torch.Tensor, *, block_size: int, window: int, scale: float,
                     max_kv_len: int, n_splits: int = 0, generic: bool = False) -> None:
    """out[row, head] = soft-max(q_abs . cache rows * scale) weighted latent over the row's visible positions."""
    rows, heads, R = q_abs.shape
    c_pad = out.size(2)
    _need(q_abs.is_contiguous() and out.is_contiguous() and out.shape[:2] == q_abs.shape[:2] and cache.size(1) == R and
          cache.is_contiguous() and cache.dtype == q_abs.dtype == out.dtype, "latent_attention: shapes")
    _i32(positions, rows, "positions")
    n = q_cu.numel() - 1
    _i32(q_cu, 2, "q_cu")
    _i32(block_cu, n + 1, "block_cu")
    _i32(block_table, 1, "block_table")
    a = _lib.LatentAttnArgs()
    a.q_abs, a.cache, a.out, a.positions = _p(q_abs), _p(cache), _p(out), _p(positions)
    a.q_cu, a.block_table, a.block_cu = _p(q_cu), _p(block_table), _p(block_cu)
    a.rows, a.batch, a.heads, a.c_pad, a.r_pad = rows, n, heads, c_pad, R - c_pad
    a.block_size, a.window, a.max_kv_len, a.n_splits = block_size, int(window), int(max_kv_len), int(n_splits)
    a.scale, a.dtype, a.generic = float(scale), _code(q_abs), int(generic)
    L = _lib.latent_lib()
    need = L.slm_latent_attn_workspace_bytes(C.byref(a))
    if need:
        ws = reserve_workspace(need, q_abs.device)
        a.workspace, a.workspace_bytes = ws.data_ptr(), ws.numel()
    latent_check(L.slm_latent_attn(C.byref(a), _stream()), "slm_latent_attn")


def latent_gather(cache: torch.Tensor, slots: torch.Tensor) -> torch.Tensor:
    """cache rows of `slots`, contiguous."""
    n = slots.numel()
    _i32(slots, n, "slots")
    out = torch.empty(n, cache.size(1), dtype=cache.dtype, device=cache.device)
    latent_check(_lib.latent_lib().slm_latent_gather(_p(out), _p(cache), _p(slots), n, cache.size(1) * cache.element_size(), _stream()),
                 "slm_latent_gather")
    return out


def latent_prefill_supported(q_dim: int, r_pad: int, v_pad: int) -> bool:
    return bool(_lib.latent_lib().slm_latent_prefill_supported(q_dim, r_pad, v_pad))


def latent_prefill(proj: torch.Tensor, ctx: torch.Tensor, kv: torch.Tensor, out: torch.Tensor, tiles: torch.Tensor, *, heads: int,
                   q_dim: int, c_pad: int, v_pad: int, gate_off: int, window: int, scale: float) -> None:
    """Causal, windowed attention of the portions' query rows over their expanded context; see slm_latent.h."""
    r_pad = ctx.size(1) - c_pad
    _need(proj.dtype == ctx.dtype == kv.dtype == out.dtype == torch.bfloat16, "latent_prefill: bfloat16")
    _need(ctx.is_contiguous() and kv.is_contiguous() and kv.shape == (ctx.size(0), heads * (q_dim + v_pad)), "latent_prefill: context")
    _need(tiles.dim() == 2 and tiles.size(1) == 6, "latent_prefill: tiles")
    _i32(tiles, tiles.numel(), "tiles")
    a = _lib.LatentPrefillArgs()
    a.q, a.ctx, a.kv, a.gate, a.out, a.tiles = _p(proj), _p(ctx), _p(kv), _p(proj), _p(out), _p(tiles)
    a.ld_q, a.ld_out, a.n_rows, a.n_ctx, a.gate_off = proj.stride(0), out.stride(0), proj.size(0), ctx.size(0), gate_off
    a.n_tiles, a.heads, a.q_dim, a.c_pad, a.r_pad, a.v_pad = tiles.size(0), heads, q_dim, c_pad, r_pad, v_pad
    a.window, a.scale = int(window), float(scale)
    latent_check(_lib.latent_lib().slm_latent_prefill(C.byref(a), _stream()), "slm_latent_prefill")
