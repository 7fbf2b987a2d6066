// latent_cache.hip -- the latent cache: append (latent RMS norm + rotation, fused) and gather.
// Cache row of a token: [c_pad] normed latent | [r_pad] rotated key part shared by all heads, zero padded.
// Bound: HBM, trivial.
#include "latent_common.h"

namespace slm {

// One workgroup per token.  V elements at a time where the widths allow it (rank, rot / 2 multiples of V).
template <typename E, int V>
__global__ void __launch_bounds__(256) latent_append_kernel(const slm_latent_append_args a) {
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int64_t row = blockIdx.x;
  E* pr = reinterpret_cast<E*>(a.proj) + row * a.ld_proj;
  E* cr = reinterpret_cast<E*>(a.cache) + (int64_t)a.slots[row] * (a.c_pad + a.r_pad);
  const int half = a.rot / 2;
  const float* cs = a.cos_sin + (int64_t)a.positions[row] * a.rot;

  // pairs (j, j + half), j .. j + V - 1, of src -> x, y
  auto rotate = [&](const E* src, int j, float (&x)[V], float (&y)[V]) {
    float u[V], v[V], c[V], s[V];
    load_f32<V>(src + j, u);
    load_f32<V>(src + half + j, v);
    load_f32<V>(cs + j, c);
    load_f32<V>(cs + half + j, s);
#pragma unroll
    for (int k = 0; k < V; ++k) {
      x[k] = u[k] * c[k] - v[k] * s[k];
      y[k] = v[k] * c[k] + u[k] * s[k];
    }
  };

  // the rotated part of every query head, in place and (absorbed rows) into q_abs
  const int hd = a.q_dim + a.q_rot, row_w = a.c_pad + a.r_pad, hv = half / V;
  E* qa = a.q_abs && row < a.abs_rows ? reinterpret_cast<E*>(a.q_abs) + row * (int64_t)a.heads * row_w : nullptr;
  for (int i = tid; i < a.heads * hv; i += 256) {
    const int h = i / hv, j = i % hv * V;
    E* q = pr + h * hd + a.q_dim;
    float x[V], y[V];
    rotate(q, j, x, y);
    store_f32<V>(q + j, x);
    store_f32<V>(q + half + j, y);
    if (qa) {
      store_f32<V>(qa + (int64_t)h * row_w + a.c_pad + j, x);
      store_f32<V>(qa + (int64_t)h * row_w + a.c_pad + half + j, y);
    }
  }
  if (qa) {
    const int pad = a.r_pad - a.rot;
    for (int i = tid; i < a.heads * pad; i += 256) qa[(int64_t)(i / pad) * row_w + a.c_pad + a.rot + i % pad] = (E)0.f;
  }

  // the shared key part
  for (int i = tid * V; i < half; i += 256 * V) {
    float x[V], y[V];
    rotate(pr + a.off_r, i, x, y);
    store_f32<V>(cr + a.c_pad + i, x);
    store_f32<V>(cr + a.c_pad + half + i, y);
  }
  for (int i = a.rot + tid; i < a.r_pad; i += 256) cr[a.c_pad + i] = (E)0.f;

  // latent: x / sqrt(mean(x^2) + eps) * w over `rank` entries
  const E* lat = pr + a.off_c;
  float ss = 0.f;
  for (int i = tid * V; i < a.rank; i += 256 * V) {
    float v[V];
    load_f32<V>(lat + i, v);
#pragma unroll
    for (int k = 0; k < V; ++k) ss = __builtin_fmaf(v[k], v[k], ss);
  }
  const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)a.rank + a.eps);
  for (int i = tid * V; i < a.rank; i += 256 * V) {
    float v[V], w[V];
    load_f32<V>(lat + i, v);
    load_f32<V>(a.norm_weight + i, w);
#pragma unroll
    for (int k = 0; k < V; ++k) v[k] = v[k] * rs * w[k];
    store_f32<V>(cr + i, v);
  }
  for (int i = a.rank + tid; i < a.c_pad; i += 256) cr[i] = (E)0.f;
}

__global__ void __launch_bounds__(256) latent_gather_kernel(u32x4* __restrict__ out, const u32x4* __restrict__ cache,
                                                            const int32_t* __restrict__ slots, int64_t n_chunks, int chunks) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n_chunks) return;
  const int64_t r = i / chunks;
  out[i] = cache[(int64_t)slots[r] * chunks + i % chunks];
}

}  // namespace slm

using namespace slm;

extern "C" SLM_API int slm_latent_append(const slm_latent_append_args* a, void* stream) {
  if (!a || !a->proj || !a->cache || !a->norm_weight || !a->cos_sin || !a->positions || !a->slots || a->rows < 0 ||
      a->heads < 1 || a->q_dim < 0 || a->rot < 2 || a->rot % 2 || a->rot > a->r_pad || a->rot > a->q_rot ||
      a->rank < 1 || a->rank > a->c_pad || a->abs_rows < 0 || a->abs_rows > a->rows ||
      a->ld_proj < (int64_t)a->heads * (a->q_dim + a->q_rot) || a->off_c < 0 || a->off_r < 0 ||
      a->off_c + a->rank > a->ld_proj || a->off_r + a->rot > a->ld_proj)
    return SLM_ERR_INVALID_ARG;
  if (a->rows == 0) return SLM_OK;
  hip_clear_error();
  const dim3 grid((unsigned)a->rows);
  hipStream_t st = (hipStream_t)stream;
  const bool v4 = a->rank % 4 == 0 && a->rot % 8 == 0 && a->q_dim % 4 == 0 && a->q_rot % 4 == 0 && a->ld_proj % 4 == 0 &&
                  a->off_c % 4 == 0 && a->off_r % 4 == 0 && a->c_pad % 4 == 0 && a->r_pad % 4 == 0 && aligned16(a->proj) &&
                  aligned16(a->cache) && aligned16(a->q_abs) && aligned16(a->norm_weight) && aligned16(a->cos_sin);
  if (a->dtype == SLM_BF16) {
    if (v4) latent_append_kernel<bf16, 4><<<grid, dim3(256), 0, st>>>(*a);
    else latent_append_kernel<bf16, 1><<<grid, dim3(256), 0, st>>>(*a);
  } else if (a->dtype == SLM_F32) {
    if (v4) latent_append_kernel<float, 4><<<grid, dim3(256), 0, st>>>(*a);
    else latent_append_kernel<float, 1><<<grid, dim3(256), 0, st>>>(*a);
  } else {
    return SLM_ERR_UNSUPPORTED;
  }
  return hip_check_launch();
}

extern "C" SLM_API int slm_latent_gather(void* out, const void* cache, const int32_t* slots, int64_t n, int64_t row_bytes,
                                         void* stream) {
  if (!out || !cache || !slots || n < 0 || row_bytes <= 0 || row_bytes % 16) return SLM_ERR_INVALID_ARG;
  if (!aligned16(out) || !aligned16(cache)) return SLM_ERR_ALIGNMENT;
  if (n == 0) return SLM_OK;
  const int chunks = (int)(row_bytes / 16);
  const int64_t total = n * chunks;
  hip_clear_error();
  latent_gather_kernel<<<dim3((unsigned)((total + 255) / 256)), dim3(256), 0, (hipStream_t)stream>>>(
      (u32x4*)out, (const u32x4*)cache, slots, total, chunks);
  return hip_check_launch();
}
