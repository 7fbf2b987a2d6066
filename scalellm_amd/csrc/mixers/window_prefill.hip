// window_prefill.hip -- windowed grouped-query attention of prompt portions on MFMA: kept first tokens, capped scores,
// a sink.  The portion's context is a list of cache slots (kept positions, then the window of its first row onwards).
//
// Work item: one workgroup = (tile of 128 query rows of one sequence, head); four waves of 32 query rows.
//   S^T[64 keys x 32 q] = K Q^T    v_mfma_f32_32x32x16_bf16, A = K rows from LDS (row stride an odd number of 16-byte
//                                  units), B = Q rows in registers
//   cap, mask, soft-max            a lane holds 32 scores of ONE query row: register reductions + one lane-half exchange
//   O^T[v x 32 q] += V^T P^T       P^T stays in registers: the C-fragment key order {4h + e, 8 + 4h + e} is the
//                                  contraction order; V^T comes out of the row-major tile by the transpose read
// The next tile travels global -> registers while this one is consumed, its slots one tile further ahead.  Key tiles are
// those of the kept tokens, then those of the tile's own window.  Bound: MFMA.
#include "window_common.h"

namespace slm {

typedef short wtr_v4 __attribute__((ext_vector_type(4)));
typedef short wtr_v8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) wtr_v4 wtr_lds_v4;

template <int DQ, int VP>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DQ + VP >= 384 ? 1 : 2)))
window_prefill_kernel(const slm_window_prefill_args a) {
  constexpr int KT = 64;
  constexpr int KLS = DQ * 2 + 16;
  constexpr int VLS = VP * 2 + ((VP * 2) % 128 == 0 ? 64 : 0);
  constexpr int QS = DQ / 16, DT = VP / 32;
  constexpr int KCH = DQ / 8, VCH = VP / 8;          // 16-byte chunks of a row
  constexpr int NK = KT * KCH / 256, NV = KT * VCH / 256;
  static_assert(KT * KCH % 256 == 0 && KT * VCH % 256 == 0, "whole chunks per thread");
  __shared__ __attribute__((aligned(16))) char k_lds[KT * KLS];
  __shared__ __attribute__((aligned(16))) char v_lds[KT * VLS];
  __shared__ int slot_lds[2][KT];

  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l31 = lane & 31, hh = lane >> 5;
  // heads fastest: the query tiles of one head stay on one XCD (heads % 8 == 0) and share its keys in L2
  const int head = blockIdx.x % a.heads, g = head / (a.heads / a.kv_heads);
  const int32_t* td = a.tiles + 7 * (blockIdx.x / a.heads);
  const int row0 = td[0], n_rows = td[1], ctx0 = td[2], ctx_len = td[3], kept = td[4], first = td[5], pos0 = td[6];
  const int shift = first - kept;                      // position = index + shift behind the kept tokens

  // context indexes the tile needs: [0, n_keep) and [lo, hi)
  const int hi = min(ctx_len, pos0 + n_rows - shift);
  const int n_keep = a.window > 0 ? min(max(a.keep_first, 0), hi) : 0;
  int lo = a.window > 0 ? max(n_keep, pos0 - a.window + 1 - shift) : 0;
  int n_head = (n_keep + KT - 1) / KT;                 // tiles of the kept tokens
  if (lo == n_keep) lo = 0, n_head = 0;                // (one range)
  const int n_tiles = n_head + (hi - lo + KT - 1) / KT;
  auto tile_start = [&](int t) { return t < n_head ? t * KT : lo + (t - n_head) * KT; };
  auto tile_end = [&](int t) { return t < n_head ? n_keep : hi; };

  // this lane's query row
  const int qi = min(wave * 32 + l31, n_rows - 1);
  bf16x8_t qf[QS];
  {
    const bf16* q = reinterpret_cast<const bf16*>(a.q) + (int64_t)(row0 + qi) * a.ld_q + (int64_t)head * DQ + 8 * hh;
#pragma unroll
    for (int s = 0; s < QS; ++s) qf[s] = *reinterpret_cast<const bf16x8_t*>(q + 16 * s);
  }
  // in context indexes: the row's own, the first one its window holds
  const int qidx = pos0 + qi - shift;
  const int klo = a.window > 0 ? qidx - a.window + 1 : 0;
  const int wq0 = pos0 - shift + min(wave * 32, n_rows - 1), wq1 = pos0 - shift + min(wave * 32 + 31, n_rows - 1);

  const bf16* kc = reinterpret_cast<const bf16*>(a.key_cache) + (int64_t)g * DQ;
  const bf16* vc = reinterpret_cast<const bf16*>(a.value_cache) + (int64_t)g * VP;
  const int64_t k_w = (int64_t)a.kv_heads * DQ, v_w = (int64_t)a.kv_heads * VP;

  auto slot_of = [&](int t) { return a.slots[ctx0 + min(tile_start(t) + lane, tile_end(t) - 1)]; };
  u32x4 ks[NK], vs[NV];
  auto load_tile = [&](int b) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int idx = tid + 256 * i;
      ks[i] = *reinterpret_cast<const u32x4*>(kc + (int64_t)slot_lds[b][idx / KCH] * k_w + 8 * (idx % KCH));
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int idx = tid + 256 * i;
      vs[i] = *reinterpret_cast<const u32x4*>(vc + (int64_t)slot_lds[b][idx / VCH] * v_w + 8 * (idx % VCH));
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
  // log2 units: without a cap scale2 * s, with one cap2 * tanh(s * scale / softcap)
  const bool capped = a.softcap > 0.f;
  const float scale2 = a.scale * LOG2E_F, cap2 = a.softcap * LOG2E_F, cap_in = capped ? 2.0f * LOG2E_F * a.scale / a.softcap : 0.f;

  // transpose read: key 4 hh + (lane % 16) / 4, columns 16 (lane / 16 % 2) + 4 (lane % 4)
  const uint32_t tr_base = (uint32_t)(uintptr_t)v_lds +
                           (uint32_t)((4 * hh + ((lane & 15) >> 2)) * VLS + ((lane >> 4) & 1) * 32 + (lane & 3) * 8);
  const char* k_base = k_lds + l31 * KLS + hh * 16;

  if (wave == 0) {
    slot_lds[0][lane] = slot_of(0);
    slot_lds[1][lane] = slot_of(min(1, n_tiles - 1));
  }
  __syncthreads();
  load_tile(0);
  for (int t = 0; t < n_tiles; ++t) {
    const int k0 = tile_start(t), k_end = tile_end(t);
    int next_slot = 0;
    if (wave == 0) next_slot = slot_of(min(t + 2, n_tiles - 1));
    store_tile();
    lds_barrier();
    if (t + 1 < n_tiles) load_tile((t + 1) & 1);
    // tiles no row of this wave sees (past its diagonal, before its window) are skipped
    const bool seen = k0 <= wq1 && (a.window <= 0 || k0 < n_keep || k0 + KT > wq0 - a.window + 1);
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
      if (capped) {
#pragma unroll
        for (int n = 0; n < 2; ++n)
#pragma unroll
          for (int r = 0; r < 16; ++r)
            s[n][r] = cap2 * (1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + fast_exp2(s[n][r] * cap_in)));
      } else {
#pragma unroll
        for (int n = 0; n < 2; ++n)
#pragma unroll
          for (int r = 0; r < 16; ++r) s[n][r] *= scale2;
      }
      const bool inside = k0 + KT - 1 <= wq0 && k0 + KT <= k_end && (a.window <= 0 || k0 >= wq1 - a.window + 1);
      if (!inside) {
#pragma unroll
        for (int n = 0; n < 2; ++n)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int key = k0 + 32 * n + 8 * (r >> 2) + 4 * hh + (r & 3);
            if (key > qidx || key >= k_end || (key < klo && key >= n_keep)) s[n][r] = -INFINITY;
          }
      }
      float mx = s[0][0];
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int r = 0; r < 16; ++r) mx = fmaxf(mx, s[n][r]);
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float m_new = fmaxf(m_run, mx);
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
          const float e0 = fast_exp2(s[f >> 1][r] - m_new);
          const float e1 = fast_exp2(s[f >> 1][r + 1] - m_new);
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
          const wtr_v4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((wtr_lds_v4*)(uintptr_t)ad);
          const wtr_v4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((wtr_lds_v4*)(uintptr_t)(ad + 8 * VLS));
          const wtr_v8 v = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
          o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, v), pf[f], o[d], 0, 0, 0);
        }
    }
    if (wave == 0) slot_lds[t & 1][lane] = next_slot;   // (tile t's own slots were last read an iteration ago)
    lds_barrier();
  }

  l_run += __shfl_xor(l_run, 32, 64);
  if (wave * 32 + l31 >= n_rows) return;
  float f = 1.0f;
  if (a.sink) {
    const float s2 = a.sink[head] * LOG2E_F, top = fmaxf(m_run, s2);
    f = fast_exp2(m_run - top);
    l_run = l_run * f + fast_exp2(s2 - top);
  }
  const float w = a.out_scale * f / l_run;
  bf16* out = reinterpret_cast<bf16*>(a.out) + (int64_t)(row0 + qi) * a.ld_out + head * VP + 4 * hh;
#pragma unroll
  for (int d = 0; d < DT; ++d)
#pragma unroll
    for (int r = 0; r < 16; r += 4)
      *reinterpret_cast<u32x2*>(out + 32 * d + 2 * r) = u32x2{pack2<bf16_tag>(o[d][r] * w, o[d][r + 1] * w),
                                                              pack2<bf16_tag>(o[d][r + 2] * w, o[d][r + 3] * w)};
}

static bool wp_width(int w) { return w == 64 || w == 96 || w == 128 || w == 192 || w == 256; }
template <int DQ, int VP>
static void wp_launch(const slm_window_prefill_args& a, hipStream_t st) {
  window_prefill_kernel<DQ, VP><<<dim3((unsigned)((int64_t)a.n_tiles * a.heads)), dim3(256), 0, st>>>(a);
}
template <int DQ>
static void wp_v(const slm_window_prefill_args& a, hipStream_t st) {
  switch (a.v_pad) {
    case 64: wp_launch<DQ, 64>(a, st); break;
    case 96: wp_launch<DQ, 96>(a, st); break;
    case 128: wp_launch<DQ, 128>(a, st); break;
    case 192: wp_launch<DQ, 192>(a, st); break;
    default: wp_launch<DQ, 256>(a, st);
  }
}

}  // namespace slm

using namespace slm;

extern "C" SLM_API int slm_window_prefill_supported(int32_t d_pad, int32_t v_pad) { return wp_width(d_pad) && wp_width(v_pad) ? 1 : 0; }
extern "C" SLM_API int slm_window_prefill(const slm_window_prefill_args* a, void* stream) {
  if (!a || !a->q || !a->key_cache || !a->value_cache || !a->out || !a->slots || !a->tiles || a->n_tiles < 0 || a->heads < 1 ||
      a->kv_heads < 1 || a->heads % a->kv_heads || a->n_rows < 0 || a->n_ctx < 0 || (int64_t)a->n_tiles * a->heads > 0x7fffffff)
    return SLM_ERR_INVALID_ARG;
  if (!slm_window_prefill_supported(a->d_pad, a->v_pad)) return SLM_ERR_UNSUPPORTED;
  if (a->ld_q < (int64_t)a->heads * a->d_pad || a->ld_out < (int64_t)a->heads * a->v_pad || a->ld_q % 8 || a->ld_out % 4 ||
      !aligned16(a->q) || !aligned16(a->key_cache) || !aligned16(a->value_cache) || !aligned16(a->out))
    return SLM_ERR_ALIGNMENT;
  if (a->n_tiles == 0) return SLM_OK;
  hip_clear_error();
  switch (a->d_pad) {
    case 64: wp_v<64>(*a, (hipStream_t)stream); break;
    case 96: wp_v<96>(*a, (hipStream_t)stream); break;
    case 128: wp_v<128>(*a, (hipStream_t)stream); break;
    case 192: wp_v<192>(*a, (hipStream_t)stream); break;
    default: wp_v<256>(*a, (hipStream_t)stream);
  }
  return hip_check_launch();
}
