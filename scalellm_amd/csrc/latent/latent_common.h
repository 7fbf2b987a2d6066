// latent_common.h -- shared helpers of libslm_latent: element access by dtype, reductions.
#pragma once
#include "common.h"
#include "slm_latent.h"

namespace slm {

typedef __bf16 bf16;
typedef uint32_t u32x4u __attribute__((ext_vector_type(4)));

template <typename E>
__device__ __forceinline__ float to_f32(E v) { return (float)v; }

// N consecutive elements as fp32 (N * sizeof(E) bytes aligned)
template <typename E, int N>
struct Vec { E v[N]; };
template <int N>
__device__ __forceinline__ void load_f32(const float* p, float (&o)[N]) {
  const Vec<float, N> t = *reinterpret_cast<const Vec<float, N>*>(p);
#pragma unroll
  for (int i = 0; i < N; ++i) o[i] = t.v[i];
}
template <int N>
__device__ __forceinline__ void load_f32(const bf16* p, float (&o)[N]) {
  typedef bf16 vec_t __attribute__((ext_vector_type(N)));
  const vec_t t = *reinterpret_cast<const vec_t*>(p);
#pragma unroll
  for (int i = 0; i < N; ++i) o[i] = (float)t[i];
}
template <>
__device__ __forceinline__ void load_f32<1>(const float* p, float (&o)[1]) { o[0] = *p; }
template <>
__device__ __forceinline__ void load_f32<1>(const bf16* p, float (&o)[1]) { o[0] = (float)*p; }
template <>
__device__ __forceinline__ void load_f32<4>(const float* p, float (&o)[4]) {
  const f32x4 t = *reinterpret_cast<const f32x4*>(p);
  o[0] = t.x; o[1] = t.y; o[2] = t.z; o[3] = t.w;
}
template <int N>
__device__ __forceinline__ void store_f32(float* p, const float (&o)[N]) {
  if constexpr (N == 4) *reinterpret_cast<f32x4*>(p) = f32x4{o[0], o[1], o[2], o[3]};
  else
#pragma unroll
    for (int i = 0; i < N; ++i) p[i] = o[i];
}
template <int N>
__device__ __forceinline__ void store_f32(bf16* p, const float (&o)[N]) {
  if constexpr (N == 4) *reinterpret_cast<u32x2*>(p) = u32x2{pack2<bf16_tag>(o[0], o[1]), pack2<bf16_tag>(o[2], o[3])};
  else
#pragma unroll
    for (int i = 0; i < N; ++i) p[i] = (bf16)o[i];
}

__device__ __forceinline__ float wave_sum(float v) { return group_sum<64>(v); }
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = 32; o >= 1; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}
// over a workgroup of 256; `tmp` = 4 floats of LDS, reusable after the call
__device__ __forceinline__ float block_sum256(float v, float* tmp) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) tmp[threadIdx.x >> 6] = v;
  __syncthreads();
  return tmp[0] + tmp[1] + tmp[2] + tmp[3];
}
__device__ __forceinline__ float block_max256(float v, float* tmp) {
  v = wave_max(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) tmp[threadIdx.x >> 6] = v;
  __syncthreads();
  return fmaxf(fmaxf(tmp[0], tmp[1]), fmaxf(tmp[2], tmp[3]));
}

__device__ __forceinline__ float sigmoid_f32(float x) { return 1.0f / (1.0f + __expf(-x)); }
__device__ __forceinline__ float clamped_glu_f32(float g, float u, float limit, float alpha, float shift) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f32(alpha * g) * (u + shift);
}

// sequence of a query row: the last s with q_cu[s] <= row (batch >= 1)
__device__ __forceinline__ int seq_of_row(const int32_t* q_cu, int batch, int row) {
  int lo = 0, hi = batch - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (q_cu[mid] <= row) lo = mid; else hi = mid - 1;
  }
  return lo;
}

constexpr float LOG2E_F = 1.4426950408889634f;
constexpr float M_INIT_F = -1.0e30f;

// barrier for LDS traffic only: outstanding global loads (register prefetch) stay in flight
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

}  // namespace slm
