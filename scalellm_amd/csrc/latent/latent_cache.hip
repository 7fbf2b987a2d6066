// latent_cache.hip -- the latent cache: append (latent RMS norm + rotation, fused) and gather.
// Cache row of a token: [c_pad] normed latent | [r_pad] rotated key part shared by all heads, zero padded.
// Bound: HBM, trivial.
#include "latent_common.h"

namespace slm {

// One workgroup per token.
template <typename E>
__global__ void __launch_bounds__(256) latent_append_kernel(const slm_latent_append_args a) {
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const int64_t row = blockIdx.x;
  E* pr = reinterpret_cast<E*>(a.proj) + row * a.ld_proj;
  E* cr = reinterpret_cast<E*>(a.cache) + (int64_t)a.slots[row] * (a.c_pad + a.r_pad);
  const int half = a.rot / 2;
  const float* cs = a.cos_sin + (int64_t)a.positions[row] * a.rot;

  // latent: x / sqrt(mean(x^2) + eps) * w over `rank` entries
  const E* lat = pr + a.off_c;
  float ss = 0.f;
  for (int i = tid; i < a.rank; i += 256) {
    const float v = to_f32(lat[i]);
    ss = __builtin_fmaf(v, v, ss);
  }
  const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)a.rank + a.eps);
  for (int i = tid; i < a.c_pad; i += 256) cr[i] = i < a.rank ? (E)(to_f32(lat[i]) * rs * a.norm_weight[i]) : (E)0.f;

  // the shared key part: pairs (i, i + half)
  const E* kr = pr + a.off_r;
  for (int i = tid; i < half; i += 256) {
    const float u = to_f32(kr[i]), v = to_f32(kr[i + half]), c = cs[i], s = cs[half + i];
    cr[a.c_pad + i] = (E)(u * c - v * s);
    cr[a.c_pad + half + i] = (E)(v * c + u * s);
  }
  for (int i = a.rot + tid; i < a.r_pad; i += 256) cr[a.c_pad + i] = (E)0.f;

  // the rotated part of every query head, in place and (absorbed rows) into q_abs
  const int hd = a.q_dim + a.q_rot, row_w = a.c_pad + a.r_pad;
  E* qa = a.q_abs && row < a.abs_rows ? reinterpret_cast<E*>(a.q_abs) + row * (int64_t)a.heads * row_w : nullptr;
  for (int i = tid; i < a.heads * half; i += 256) {
    const int h = i / half, j = i % half;
    E* q = pr + h * hd + a.q_dim;
    const float u = to_f32(q[j]), v = to_f32(q[j + half]), c = cs[j], s = cs[half + j];
    const E x = (E)(u * c - v * s), y = (E)(v * c + u * s);
    q[j] = x;
    q[j + half] = y;
    if (qa) {
      qa[(int64_t)h * row_w + a.c_pad + j] = x;
      qa[(int64_t)h * row_w + a.c_pad + half + j] = y;
    }
  }
  if (qa) {
    const int pad = a.r_pad - a.rot;
    for (int i = tid; i < a.heads * pad; i += 256) qa[(int64_t)(i / pad) * row_w + a.c_pad + a.rot + i % pad] = (E)0.f;
  }
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
  if (a->dtype == SLM_BF16) latent_append_kernel<bf16><<<grid, dim3(256), 0, (hipStream_t)stream>>>(*a);
  else if (a->dtype == SLM_F32) latent_append_kernel<float><<<grid, dim3(256), 0, (hipStream_t)stream>>>(*a);
  else return SLM_ERR_UNSUPPORTED;
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
