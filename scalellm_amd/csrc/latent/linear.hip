// linear.hip -- y = x W^T for few rows (decode batches, the vocabulary projection of the sampled rows), and
// for every row count in 32-bit.  Bound: the HBM stream of W.
//
// A workgroup of four waves owns NT blocks of 16 output columns and MT blocks of 16 rows of x and splits K
// over its waves (and over blockIdx for SLABS).  Per step of 64 a lane (r = lane % 16, g = lane / 16) reads
// the 16 consecutive k of row r that start at 16 g -- the four lane groups of a row read one whole 128-byte
// line in bf16 -- and feeds them to the MFMAs in an order of k that is the same for both operands, so no
// shuffle is needed.  The waves' partial tiles meet in LDS; the epilogue runs there.
#include "latent_common.h"

namespace slm {

template <typename E>
struct KStep;  // 64 k of one 16-row block: what a lane holds
template <>
struct KStep<bf16> {
  bf16x8_t v[2];
  __device__ __forceinline__ void load(const bf16* p) {
    v[0] = *reinterpret_cast<const bf16x8_t*>(p);
    v[1] = *reinterpret_cast<const bf16x8_t*>(p + 8);
  }
  __device__ __forceinline__ void zero() {
    v[0] = __builtin_bit_cast(bf16x8_t, u32x4{0u, 0u, 0u, 0u});
    v[1] = v[0];
  }
  static __device__ __forceinline__ f32x4 mma(const KStep& a, const KStep& b, f32x4 c) {
    c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v[0], b.v[0], c, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v[1], b.v[1], c, 0, 0, 0);
  }
};
template <>
struct KStep<float> {
  f32x4 v[4];
  __device__ __forceinline__ void load(const float* p) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = *reinterpret_cast<const f32x4*>(p + 4 * i);
  }
  __device__ __forceinline__ void zero() {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  static __device__ __forceinline__ f32x4 mma(const KStep& a, const KStep& b, f32x4 c) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[i][j], b.v[i][j], c, 0, 0, 0);
    return c;
  }
};

// GLU: the NT blocks are NT / 2 pairs (gate block, up block half columns further)
template <typename E, int MT, int NT, int U, int EPI>
__global__ void __launch_bounds__(256) linear_kernel(const slm_linear_args a) {
  constexpr bool GLU = EPI == SLM_LIN_GLU;
  constexpr int NOUT = GLU ? NT / 2 : NT;  // output column blocks
  static_assert(!GLU || NT % 2 == 0, "gate / up pairs");
  __shared__ f32x4 red[4][NT * MT][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r16 = lane & 15, g = lane >> 4;
  const int z = blockIdx.z;
  const int item = z / a.n_splits, split = z % a.n_splits;
  const int64_t half = a.N / 2;
  const int64_t n_out = GLU ? half : a.N;
  const int64_t n0 = (int64_t)blockIdx.x * (16 * NOUT), m0 = (int64_t)blockIdx.y * (16 * MT);

  const E* wp[NT];
  const E* xp[MT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    int64_t n = GLU ? n0 + 16 * (t >> 1) : n0 + 16 * t;
    n = min(n, n_out - 16) + r16 + (GLU ? (t & 1) * half : 0);  // (a block past the end re-reads the last: not stored)
    wp[t] = reinterpret_cast<const E*>(a.w) + item * a.w_batch + n * a.ldw + 16 * g;
  }
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int64_t m = min(m0 + 16 * t + r16, a.M - 1);
    xp[t] = reinterpret_cast<const E*>(a.x) + item * a.x_batch + m * a.ldx + 16 * g;
  }
  f32x4 acc[NT][MT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int u = 0; u < MT; ++u) acc[t][u] = f32x4{0.f, 0.f, 0.f, 0.f};

  const int steps = (int)(a.K >> 6);
  const int per = (steps + a.n_splits - 1) / a.n_splits;
  const int s0 = split * per, s1 = min(steps, s0 + per);
  int s = s0 + wave;
  for (; s + 4 * (U - 1) < s1; s += 4 * U) {
    KStep<E> w[U][NT], x[U][MT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int64_t k = (int64_t)(s + 4 * u) << 6;
#pragma unroll
      for (int t = 0; t < NT; ++t) w[u][t].load(wp[t] + k);
#pragma unroll
      for (int t = 0; t < MT; ++t) x[u][t].load(xp[t] + k);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int v = 0; v < MT; ++v) acc[t][v] = KStep<E>::mma(w[u][t], x[u][v], acc[t][v]);
  }
  if constexpr (U > 1) {
    for (; s < s1; s += 4) {
      const int64_t k = (int64_t)s << 6;
      KStep<E> x[MT];
#pragma unroll
      for (int t = 0; t < MT; ++t) x[t].load(xp[t] + k);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        KStep<E> w;
        w.load(wp[t] + k);
#pragma unroll
        for (int v = 0; v < MT; ++v) acc[t][v] = KStep<E>::mma(w, x[v], acc[t][v]);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int v = 0; v < MT; ++v) red[wave][t * MT + v][lane] = acc[t][v];
  __syncthreads();

  // thread = (column n of 16, row m of 16) of every tile; C layout: row n = 4 (lane / 16) + reg, column m = lane % 16
  const int n = tid & 15, m = tid >> 4;
  const int src = (n >> 2) * 16 + m, reg = n & 3;
  auto total = [&](int t) {
    float v = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) v += reinterpret_cast<const float*>(&red[w][t][src])[reg];
    return v;
  };
#pragma unroll
  for (int t = 0; t < NOUT; ++t) {
    const int64_t nn = n0 + 16 * t + n;
    if (nn >= n_out) continue;
#pragma unroll
    for (int v = 0; v < MT; ++v) {
      const int64_t mm = m0 + 16 * v + m;
      if (mm >= a.M) continue;
      if constexpr (EPI == SLM_LIN_SLABS) {
        reinterpret_cast<float*>(a.y)[((int64_t)split * a.M + mm) * a.ldy + nn] = total(t * MT + v);
      } else if constexpr (EPI == SLM_LIN_F32) {
        reinterpret_cast<float*>(a.y)[item * a.y_batch + mm * a.ldy + nn] = a.alpha * total(t * MT + v);
      } else if constexpr (EPI == SLM_LIN_GLU) {
        reinterpret_cast<E*>(a.y)[mm * a.ldy + nn] =
            (E)clamped_glu_f32(total(2 * t * MT + v), total((2 * t + 1) * MT + v), a.limit, a.glu_alpha, a.glu_shift);
      } else if constexpr (EPI == SLM_LIN_GATE) {
        const float gl = to_f32(reinterpret_cast<const E*>(a.gate)[mm * a.ld_gate + item]);
        reinterpret_cast<E*>(a.y)[item * a.y_batch + mm * a.ldy + nn] = (E)(total(t * MT + v) * sigmoid_f32(gl));
      } else {
        reinterpret_cast<E*>(a.y)[item * a.y_batch + mm * a.ldy + nn] = (E)total(t * MT + v);
      }
    }
  }
}

template <typename E, int MT, int NT, int U, int EPI>
static int lin_launch(const slm_linear_args& a, hipStream_t st) {
  constexpr int NOUT = EPI == SLM_LIN_GLU ? NT / 2 : NT;
  const int64_t n_out = EPI == SLM_LIN_GLU ? a.N / 2 : a.N;
  const int64_t gx = (n_out + 16 * NOUT - 1) / (16 * NOUT), gy = (a.M + 16 * MT - 1) / (16 * MT);
  const int64_t gz = (int64_t)a.batch * a.n_splits;
  if (gx > 0x7fffffff || gy > 65535 || gz > 65535) return SLM_ERR_UNSUPPORTED;
  hip_clear_error();
  linear_kernel<E, MT, NT, U, EPI><<<dim3((unsigned)gx, (unsigned)gy, (unsigned)gz), dim3(256), 0, st>>>(a);
  return hip_check_launch();
}
// Tiles by row count: one row block streams W with many steps in flight; with more rows the reads of x weigh as much
// as those of W, and wider column blocks (where enough of them are left to fill the chip) read x less often.
template <typename E, int EPI>
static int lin_shape(const slm_linear_args& a, hipStream_t st) {
  constexpr int P = EPI == SLM_LIN_GLU ? 2 : 1;
  if constexpr (sizeof(E) == 4) {
    if (a.M <= 16) return lin_launch<E, 1, P, 1, EPI>(a, st);
    return lin_launch<E, 2, 2, 1, EPI>(a, st);
  } else {
    if (a.M <= 4) return lin_launch<E, 1, P, 8 / P, EPI>(a, st);
    if (a.M <= 16) return lin_launch<E, 1, P, 4 / P, EPI>(a, st);
    const bool wide = a.N / 64 * a.batch * a.n_splits >= 256;
    if (a.M <= 32) return wide ? lin_launch<E, 2, 4, 1, EPI>(a, st) : lin_launch<E, 2, 2, 2, EPI>(a, st);
    return wide ? lin_launch<E, 4, 4, 1, EPI>(a, st) : lin_launch<E, 4, 2, 2, EPI>(a, st);
  }
}
template <typename E>
static int lin_epi(const slm_linear_args& a, hipStream_t st) {
  switch (a.epilogue) {
    case SLM_LIN_STORE: return lin_shape<E, SLM_LIN_STORE>(a, st);
    case SLM_LIN_F32: return lin_shape<E, SLM_LIN_F32>(a, st);
    case SLM_LIN_SLABS: return lin_shape<E, SLM_LIN_SLABS>(a, st);
    case SLM_LIN_GLU: return lin_shape<E, SLM_LIN_GLU>(a, st);
    default: return lin_shape<E, SLM_LIN_GATE>(a, st);
  }
}

}  // namespace slm

using namespace slm;

extern "C" SLM_API int slm_linear(const slm_linear_args* a, void* stream) {
  if (!a || !a->x || !a->w || !a->y || a->M < 0 || a->N <= 0 || a->K <= 0 || a->K % 64 || a->N % 16 || a->batch < 1 ||
      a->n_splits < 1 || a->ldx < a->K || a->ldw < a->K || a->epilogue < 0 || a->epilogue > SLM_LIN_GATE)
    return SLM_ERR_INVALID_ARG;
  if (a->dtype != SLM_BF16 && a->dtype != SLM_F32) return SLM_ERR_UNSUPPORTED;
  const int64_t al = a->dtype == SLM_BF16 ? 8 : 4;
  if (a->ldx % al || a->ldw % al || a->x_batch % al || a->w_batch % al || !aligned16(a->x) || !aligned16(a->w))
    return SLM_ERR_ALIGNMENT;
  if (a->n_splits > 1 && (a->epilogue != SLM_LIN_SLABS || a->batch != 1)) return SLM_ERR_INVALID_ARG;
  if (a->epilogue == SLM_LIN_GLU && (a->N % 32 || a->batch != 1)) return SLM_ERR_INVALID_ARG;
  if (a->epilogue == SLM_LIN_SLABS && a->batch != 1) return SLM_ERR_INVALID_ARG;
  if (a->epilogue == SLM_LIN_GATE && !a->gate) return SLM_ERR_INVALID_ARG;
  if (a->M == 0) return SLM_OK;
  return a->dtype == SLM_BF16 ? lin_epi<bf16>(*a, (hipStream_t)stream) : lin_epi<float>(*a, (hipStream_t)stream);
}
