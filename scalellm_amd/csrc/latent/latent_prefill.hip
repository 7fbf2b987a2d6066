// latent_prefill.hip -- attention of prompt portions with latent attention in its expanded form: the latent rows
// a portion can see are gathered and multiplied by W_uk / W_uv once (a plain product), and the portion runs as
// ordinary multi-head attention with unequal query / value widths, causal and windowed, output gate fused.
//
// Work item: one workgroup = (tile of 128 query rows of one sequence, head); four waves of 32 query rows.
//   S^T[64 keys x 32 q] = K Q^T    v_mfma_f32_32x32x16_bf16, A = K rows from LDS (row stride an odd number of 16-byte
//                                  units), B = Q rows in registers.  K row = unrotated part (per head) | rotated
//                                  part (shared by the heads, out of the gathered latent rows)
//   soft-max                       a lane holds 32 scores of ONE query row: register reductions + one lane-half exchange
//   O^T[v x 32 q] += V^T P^T       P^T stays in registers: the C-fragment key order {4h + e, 8 + 4h + e} is used as the
//                                  contraction order; V^T comes out of the row-major tile by the transpose read
// The next tile travels global -> registers while this one is consumed.  Bound: MFMA.
#include "latent_common.h"

namespace slm {

typedef short trp_v4 __attribute__((ext_vector_type(4)));
typedef short trp_v8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) trp_v4 trp_lds_v4;

struct LatentPrefillK {
  slm_latent_prefill_args a;
  float scale2;
};

template <int DQ, int VP>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2)))
latent_prefill_kernel(const LatentPrefillK p) {
  constexpr int KT = 64;
  constexpr int KLS = DQ * 2 + 16;
  constexpr int VLS = VP * 2 + ((VP * 2) % 128 == 0 ? 64 : 0);
  constexpr int QS = DQ / 16, DT = VP / 32;
  constexpr int KCH = DQ / 8, VCH = VP / 8;          // 16-byte chunks of a row
  constexpr int NK = KT * KCH / 256, NV = KT * VCH / 256;
  static_assert(KT * KCH % 256 == 0 && KT * VCH % 256 == 0, "whole chunks per thread");
  __shared__ __attribute__((aligned(16))) char k_lds[KT * KLS];
  __shared__ __attribute__((aligned(16))) char v_lds[KT * VLS];

  const slm_latent_prefill_args& a = p.a;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l31 = lane & 31, hh = lane >> 5;
  // heads fastest: the query tiles of one head stay on one XCD (heads % 8 == 0) and share its keys in L2;
  // tiles come longest first from the host
  const int head = blockIdx.x % a.heads;
  const int32_t* td = a.tiles + 6 * (blockIdx.x / a.heads);
  const int row0 = td[0], n_rows = td[1], ctx0 = td[2], ctx_len = td[3], ctx_pos = td[4], pos0 = td[5];

  // visible keys of the tile, as indexes into its context
  int lo = 0, hi = min(ctx_len, pos0 + n_rows - ctx_pos);
  if (a.window > 0) lo = max(0, pos0 - a.window + 1 - ctx_pos);
  const int n_tiles = (hi - lo + KT - 1) / KT;

  // this lane's query row
  const int qi = min(wave * 32 + l31, n_rows - 1);
  const bf16* qrow = reinterpret_cast<const bf16*>(a.q) + (int64_t)(row0 + qi) * a.ld_q;
  bf16x8_t qf[QS];
  {
    const bf16* q = qrow + head * DQ + 8 * hh;
#pragma unroll
    for (int s = 0; s < QS; ++s) qf[s] = *reinterpret_cast<const bf16x8_t*>(q + 16 * s);
  }
  const int qpos = pos0 + qi - ctx_pos;  // in context indexes
  const int klo = a.window > 0 ? max(0, qpos - a.window + 1) : 0;
  // of the whole wave, for the tiles that need no mask
  const int wq0 = pos0 - ctx_pos + min(wave * 32, n_rows - 1), wq1 = pos0 - ctx_pos + min(wave * 32 + 31, n_rows - 1);

  const int q_chunks = a.q_dim / 8;
  const int64_t ctx_w = a.c_pad + a.r_pad, kv_w = (int64_t)a.heads * (a.q_dim + a.v_pad);
  const bf16* kv = reinterpret_cast<const bf16*>(a.kv) + (int64_t)head * (a.q_dim + a.v_pad);
  const bf16* ctx = reinterpret_cast<const bf16*>(a.ctx) + a.c_pad;

  u32x4 ks[NK], vs[NV];
  auto load_tile = [&](int k0) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int idx = tid + 256 * i, r = idx / KCH, c = idx % KCH;
      const int64_t key = ctx0 + min(k0 + r, hi - 1);
      const bf16* src = c < q_chunks ? kv + key * kv_w + 8 * c : ctx + key * ctx_w + 8 * (c - q_chunks);
      ks[i] = *reinterpret_cast<const u32x4*>(src);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int idx = tid + 256 * i, r = idx / VCH, c = idx % VCH;
      const int64_t key = ctx0 + min(k0 + r, hi - 1);
      vs[i] = *reinterpret_cast<const u32x4*>(kv + key * kv_w + a.q_dim + 8 * c);
    }
  };
  auto store_tile = [&]() {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int idx = tid + 256 * i;
      *reinterpret_cast<u32x4*>(k_lds + idx / KCH * KLS + idx % KCH * 16) = ks[i];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int idx = tid + 256 * i;
      *reinterpret_cast<u32x4*>(v_lds + idx / VCH * VLS + idx % VCH * 16) = vs[i];
    }
  };

  f32x16 o[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[d][r] = 0.f;
  float m_run = M_INIT_F, l_run = 0.f;

  // transpose read: key 4 hh + (lane % 16) / 4, columns 16 (lane / 16 % 2) + 4 (lane % 4)
  const uint32_t tr_base = (uint32_t)(uintptr_t)v_lds +
                           (uint32_t)((4 * hh + ((lane & 15) >> 2)) * VLS + ((lane >> 4) & 1) * 32 + (lane & 3) * 8);
  const char* k_base = k_lds + l31 * KLS + hh * 16;

  load_tile(lo);
  for (int t = 0; t < n_tiles; ++t) {
    const int k0 = lo + t * KT;
    store_tile();
    lds_barrier();
    if (t + 1 < n_tiles) load_tile(k0 + KT);
    // tiles no row of this wave sees (past its diagonal, before its window) are skipped
    const bool seen = k0 <= wq1 && (a.window <= 0 || k0 + KT > wq0 - a.window + 1);
    if (seen) {
      f32x16 s[2];
#pragma unroll
      for (int n = 0; n < 2; ++n) {
#pragma unroll
        for (int r = 0; r < 16; ++r) s[n][r] = 0.f;
#pragma unroll
        for (int i = 0; i < QS; ++i)
          s[n] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
              *reinterpret_cast<const bf16x8_t*>(k_base + 32 * n * KLS + 32 * i), qf[i], s[n], 0, 0, 0);
      }
      const bool inside = k0 + KT - 1 <= wq0 && (a.window <= 0 || k0 >= wq1 - a.window + 1);
      if (!inside) {
#pragma unroll
        for (int n = 0; n < 2; ++n)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int key = k0 + 32 * n + 8 * (r >> 2) + 4 * hh + (r & 3);
            if (key > qpos || key < klo) s[n][r] = -INFINITY;
          }
      }
      float mx = s[0][0];
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int r = 0; r < 16; ++r) mx = fmaxf(mx, s[n][r]);
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float m_new = fmaxf(m_run, mx * p.scale2);
      const float alpha = fast_exp2(m_run - m_new);
      m_run = m_new;
      float sum = 0.f;
      bf16x8_t pf[4];
#pragma unroll
      for (int f = 0; f < 4; ++f) {
        u32x4 w;
#pragma unroll
        for (int j = 0; j < 8; j += 2) {
          const int r = (f & 1) * 8 + j;
          const float e0 = fast_exp2(__builtin_fmaf(s[f >> 1][r], p.scale2, -m_new));
          const float e1 = fast_exp2(__builtin_fmaf(s[f >> 1][r + 1], p.scale2, -m_new));
          sum += e0 + e1;
          w[j >> 1] = pack2<bf16_tag>(e0, e1);
        }
        pf[f] = __builtin_bit_cast(bf16x8_t, w);
      }
      l_run = l_run * alpha + sum;
      if (__any(alpha != 1.0f)) {
#pragma unroll
        for (int d = 0; d < DT; ++d)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[d][r] *= alpha;
      }
#pragma unroll
      for (int f = 0; f < 4; ++f)
#pragma unroll
        for (int d = 0; d < DT; ++d) {
          const uint32_t ad = tr_base + (uint32_t)(16 * f * VLS + 64 * d);
          const trp_v4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((trp_lds_v4*)ad);
          const trp_v4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((trp_lds_v4*)(ad + 8 * VLS));
          const trp_v8 v = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
          o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, v), pf[f], o[d], 0, 0, 0);
        }
    }
    lds_barrier();
  }

  l_run += __shfl_xor(l_run, 32, 64);
  if (wave * 32 + l31 >= n_rows) return;
  const float w = sigmoid_f32((float)reinterpret_cast<const bf16*>(a.gate)[(int64_t)(row0 + qi) * a.ld_q + a.gate_off + head]) / l_run;
  bf16* out = reinterpret_cast<bf16*>(a.out) + (int64_t)(row0 + qi) * a.ld_out + head * VP + 4 * hh;
#pragma unroll
  for (int d = 0; d < DT; ++d)
#pragma unroll
    for (int r = 0; r < 16; r += 4)
      *reinterpret_cast<u32x2*>(out + 32 * d + 2 * r) = u32x2{pack2<bf16_tag>(o[d][r] * w, o[d][r + 1] * w),
                                                              pack2<bf16_tag>(o[d][r + 2] * w, o[d][r + 3] * w)};
}

static bool lp_ok(int dq, int vp) {
  const bool q = dq == 64 || dq == 96 || dq == 128 || dq == 160 || dq == 192 || dq == 256;
  return q && (vp == 32 || vp == 64 || vp == 128) ;
}
template <int DQ, int VP>
static void lp_launch(const LatentPrefillK& p, hipStream_t st) {
  latent_prefill_kernel<DQ, VP><<<dim3((unsigned)((int64_t)p.a.n_tiles * p.a.heads)), dim3(256), 0, st>>>(p);
}
template <int DQ>
static void lp_v(const LatentPrefillK& p, hipStream_t st) {
  switch (p.a.v_pad) {
    case 32: lp_launch<DQ, 32>(p, st); break;
    case 64: lp_launch<DQ, 64>(p, st); break;
    default: lp_launch<DQ, 128>(p, st);
  }
}

}  // namespace slm

using namespace slm;

extern "C" SLM_API int slm_latent_prefill_supported(int32_t q_dim, int32_t r_pad, int32_t v_pad) {
  return q_dim > 0 && q_dim % 8 == 0 && r_pad % 8 == 0 && lp_ok(q_dim + r_pad, v_pad) ? 1 : 0;
}
extern "C" SLM_API int slm_latent_prefill(const slm_latent_prefill_args* a, void* stream) {
  if (!a || !a->q || !a->ctx || !a->kv || !a->gate || !a->out || !a->tiles || a->n_tiles < 0 || a->heads < 1 ||
      a->n_rows < 0 || a->n_ctx < 0)
    return SLM_ERR_INVALID_ARG;
  if (!slm_latent_prefill_supported(a->q_dim, a->r_pad, a->v_pad)) return SLM_ERR_UNSUPPORTED;
  if (a->ld_q < (int64_t)a->heads * (a->q_dim + a->r_pad) || a->ld_out < (int64_t)a->heads * a->v_pad || a->ld_q % 8 ||
      a->ld_out % 4 || a->c_pad % 8 || !aligned16(a->q) || !aligned16(a->ctx) || !aligned16(a->kv) || !aligned16(a->out))
    return SLM_ERR_ALIGNMENT;
  if (a->n_tiles == 0) return SLM_OK;
  LatentPrefillK p;
  p.a = *a;
  p.scale2 = a->scale * LOG2E_F;
  hip_clear_error();
  switch (a->q_dim + a->r_pad) {
    case 64: lp_v<64>(p, (hipStream_t)stream); break;
    case 96: lp_v<96>(p, (hipStream_t)stream); break;
    case 128: lp_v<128>(p, (hipStream_t)stream); break;
    case 160: lp_v<160>(p, (hipStream_t)stream); break;
    case 192: lp_v<192>(p, (hipStream_t)stream); break;
    default: lp_v<256>(p, (hipStream_t)stream);
  }
  return hip_check_launch();
}
