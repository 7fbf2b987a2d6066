// residual_norm.hip -- the fp32 residual stream: what a sub-layer adds (or the embedding), and the norm (RMS, or
// tanh(alpha x), which needs no statistics) in front of the next projection, in one launch.  One workgroup per row; the row stays in
// registers between the sum of squares and the scaling.  Bound: HBM, trivial.
#include "latent_common.h"

namespace slm {

constexpr int RN_THREADS = 256;
constexpr int RN_STEPS = 16;  // register-resident chunks per thread

// V: elements per chunk (4 when every row start is 4-element aligned, else 1)
template <typename E, int MODE, int V>
__global__ void __launch_bounds__(RN_THREADS) residual_norm_kernel(const slm_residual_norm_args a) {
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int64_t row = blockIdx.x;
  const int width = (int)a.width;
  const int64_t src_row = (MODE == SLM_RN_PLAIN && a.row_index) ? a.row_index[row] : row;
  float* r = a.resid + src_row * a.width;
  const E* e0 = nullptr;
  const E* e1 = nullptr;
  if constexpr (MODE == SLM_RN_EMBED) {
    e0 = reinterpret_cast<const E*>(a.embed) + (int64_t)a.tokens[row] * a.ld_embed;
    if (a.pos_table) e1 = reinterpret_cast<const E*>(a.pos_table) + (int64_t)a.positions[row] * a.width;
  }
  if constexpr (MODE == SLM_RN_ADD) e0 = reinterpret_cast<const E*>(a.delta) + row * a.ld_delta;

  float x[RN_STEPS][V];
  float ss = 0.f;
#pragma unroll
  for (int s = 0; s < RN_STEPS; ++s) {
    const int i = (tid + s * RN_THREADS) * V;
    if (i < width) {
      if constexpr (MODE == SLM_RN_EMBED) {
        load_f32<V>(e0 + i, x[s]);
        if (e1) {
          float t[V];
          load_f32<V>(e1 + i, t);
#pragma unroll
          for (int j = 0; j < V; ++j) x[s][j] += t[j];
        }
#pragma unroll
        for (int j = 0; j < V; ++j) x[s][j] *= a.delta_mult;
      } else {
        load_f32<V>(r + i, x[s]);
        if constexpr (MODE == SLM_RN_ADD) {
          float t[V];
          load_f32<V>(e0 + i, t);
#pragma unroll
          for (int j = 0; j < V; ++j) x[s][j] = __builtin_fmaf(t[j], a.delta_mult, x[s][j]);
        }
        if constexpr (MODE == SLM_RN_SLABS) {
          // (all slab loads of a chunk in flight at once)
          const float* sp = a.slabs + row * a.ld_delta + i;
          float d[V];
#pragma unroll
          for (int j = 0; j < V; ++j) d[j] = 0.f;
          for (int k0 = 0; k0 < a.n_slabs; k0 += 8) {
            float t[8][V];
#pragma unroll
            for (int k = 0; k < 8; ++k)
              if (k0 + k < a.n_slabs) load_f32<V>(sp + (k0 + k) * a.slab_stride, t[k]);
#pragma unroll
            for (int k = 0; k < 8; ++k)
              if (k0 + k < a.n_slabs)
#pragma unroll
                for (int j = 0; j < V; ++j) d[j] += t[k][j];
          }
#pragma unroll
          for (int j = 0; j < V; ++j) x[s][j] = __builtin_fmaf(d[j], a.delta_mult, x[s][j]);
        }
      }
      if constexpr (MODE != SLM_RN_PLAIN) store_f32<V>(r + i, x[s]);
#pragma unroll
      for (int j = 0; j < V; ++j) ss = __builtin_fmaf(x[s][j], x[s][j], ss);
    }
  }
  if (!a.weight) return;  // (uniform: only the sum was asked for)
  const bool rms = a.norm == SLM_NORM_RMS;
  const float rs = rms ? 1.0f / sqrtf(block_sum256(ss, red) / (float)width + a.eps) : 0.f;
  E* o = reinterpret_cast<E*>(a.out) + row * a.ld_out;
#pragma unroll
  for (int s = 0; s < RN_STEPS; ++s) {
    const int i = (tid + s * RN_THREADS) * V;
    if (i < width) {
      float w[V], y[V];
      load_f32<V>(a.weight + i, w);
#pragma unroll
      for (int j = 0; j < V; ++j) y[j] = x[s][j] * rs * w[j];
      if (!rms) {
        float b[V];
        load_f32<V>(a.bias + i, b);
#pragma unroll
        for (int j = 0; j < V; ++j) y[j] = __builtin_fmaf(tanhf(a.norm_alpha * x[s][j]), w[j], b[j]);
      }
      store_f32<V>(o + i, y);
    }
  }
  for (int i = width + tid; i < (int)a.ld_out; i += RN_THREADS) o[i] = (E)0.f;
}

template <typename E>
__global__ void __launch_bounds__(256) clamped_glu_kernel(E* __restrict__ y, const E* __restrict__ gu, int64_t half4,
                                                          int64_t n4, int64_t ld_gu, int64_t ld_y, float limit, float alpha,
                                                          float shift) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n4) return;
  const int64_t row = i / half4, c = (i % half4) * 4;
  float g[4], u[4], o[4];
  load_f32<4>(gu + row * ld_gu + c, g);
  load_f32<4>(gu + row * ld_gu + half4 * 4 + c, u);
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = clamped_glu_f32(g[j], u[j], limit, alpha, shift);
  store_f32<4>(y + row * ld_y + c, o);
}

template <typename E, int MODE>
static int rn_launch(const slm_residual_norm_args& a, hipStream_t st) {
  const bool v4 = a.width % 4 == 0 && a.ld_delta % 4 == 0 && a.ld_embed % 4 == 0 && a.ld_out % 4 == 0 &&
                  a.slab_stride % 4 == 0 && aligned16(a.resid) && aligned16(a.delta) && aligned16(a.slabs) &&
                  aligned16(a.embed) && aligned16(a.pos_table) && aligned16(a.weight) && aligned16(a.bias) && aligned16(a.out);
  if (a.width > (v4 ? 4 : 1) * RN_THREADS * RN_STEPS) return SLM_ERR_UNSUPPORTED;
  hip_clear_error();
  if (v4) residual_norm_kernel<E, MODE, 4><<<dim3((unsigned)a.rows), dim3(RN_THREADS), 0, st>>>(a);
  else residual_norm_kernel<E, MODE, 1><<<dim3((unsigned)a.rows), dim3(RN_THREADS), 0, st>>>(a);
  return hip_check_launch();
}
template <typename E>
static int rn_mode(const slm_residual_norm_args& a, hipStream_t st) {
  switch (a.mode) {
    case SLM_RN_EMBED: return rn_launch<E, SLM_RN_EMBED>(a, st);
    case SLM_RN_ADD: return rn_launch<E, SLM_RN_ADD>(a, st);
    case SLM_RN_SLABS: return rn_launch<E, SLM_RN_SLABS>(a, st);
    default: return rn_launch<E, SLM_RN_PLAIN>(a, st);
  }
}

}  // namespace slm

using namespace slm;

extern "C" SLM_API const char* slm_latent_version(void) { return "slm_latent 1 (gfx950)"; }
extern "C" SLM_API const char* slm_latent_last_hip_error(void) {
  return hipGetErrorString((hipError_t)hip_last_error_slot());
}
extern "C" SLM_API const char* slm_latent_status_string(int s) {
  switch (s) {
    case SLM_OK: return "ok";
    case SLM_ERR_INVALID_ARG: return "invalid argument";
    case SLM_ERR_UNSUPPORTED: return "unsupported dtype or size";
    case SLM_ERR_WORKSPACE: return "workspace missing or too small";
    case SLM_ERR_LAUNCH: return "kernel launch failed";
    case SLM_ERR_ALIGNMENT: return "pointer or stride not aligned";
    default: return "unknown status";
  }
}

extern "C" SLM_API int slm_residual_norm(const slm_residual_norm_args* a, void* stream) {
  if (!a || a->rows < 0 || a->width <= 0 || !a->resid || a->mode < 0 || a->mode > SLM_RN_PLAIN) return SLM_ERR_INVALID_ARG;
  if (a->rows == 0) return SLM_OK;
  if (a->mode == SLM_RN_EMBED && (!a->tokens || !a->embed || a->ld_embed < a->width || (a->pos_table && !a->positions)))
    return SLM_ERR_INVALID_ARG;
  if (a->mode == SLM_RN_ADD && (!a->delta || a->ld_delta < a->width)) return SLM_ERR_INVALID_ARG;
  if (a->mode == SLM_RN_SLABS && (!a->slabs || a->n_slabs < 1 || a->ld_delta < a->width)) return SLM_ERR_INVALID_ARG;
  if (a->weight ? (!a->out || a->ld_out < a->width) : a->mode == SLM_RN_PLAIN) return SLM_ERR_INVALID_ARG;
  if (a->norm < 0 || a->norm > SLM_NORM_TANH || (a->weight && a->norm == SLM_NORM_TANH && !a->bias)) return SLM_ERR_INVALID_ARG;
  if (a->dtype == SLM_BF16) return rn_mode<bf16>(*a, (hipStream_t)stream);
  if (a->dtype == SLM_F32) return rn_mode<float>(*a, (hipStream_t)stream);
  return SLM_ERR_UNSUPPORTED;
}

extern "C" SLM_API int slm_clamped_glu(void* y, const void* gu, int64_t rows, int64_t half, int64_t ld_gu, int64_t ld_y,
                                       float limit, float glu_alpha, float glu_shift, int32_t dtype, void* stream) {
  if (!y || !gu || rows < 0 || half <= 0 || half % 4 || ld_gu < 2 * half || ld_gu % 4 || ld_y < half || ld_y % 4)
    return SLM_ERR_INVALID_ARG;
  if (!aligned16(y) || !aligned16(gu)) return SLM_ERR_ALIGNMENT;
  if (rows == 0) return SLM_OK;
  const int64_t half4 = half / 4, n4 = rows * half4;
  const dim3 grid((unsigned)((n4 + 255) / 256));
  hip_clear_error();
  if (dtype == SLM_BF16)
    clamped_glu_kernel<bf16><<<grid, dim3(256), 0, (hipStream_t)stream>>>((bf16*)y, (const bf16*)gu, half4, n4, ld_gu, ld_y, limit, glu_alpha, glu_shift);
  else if (dtype == SLM_F32)
    clamped_glu_kernel<float><<<grid, dim3(256), 0, (hipStream_t)stream>>>((float*)y, (const float*)gu, half4, n4, ld_gu, ld_y, limit, glu_alpha, glu_shift);
  else return SLM_ERR_UNSUPPORTED;
  return hip_check_launch();
}
