// window_decode.hip -- windowed grouped-query attention of single rows over the paged cache on MFMA: kept first tokens,
// capped scores, a sink.  Bound: the HBM stream of the visible keys and values.
//
// Work item: one workgroup = (row, kv head, block of 16 query heads, split of the visible keys); its four waves take tiles
// of 32 keys in turn and never meet before the end.
//   S[32 keys x 16 heads]      A = key rows straight from the cache (16 bytes per lane), B = the query heads in registers
//   O^T[v x 16 heads]          P in registers: the C-fragment key order {4 g + e, 16 + 4 g + e} is the contraction order;
//                              V^T out of a wave-private row-major LDS tile by the transpose read
// A tile's keys and values are loaded while the tile before is consumed, its slots one tile further ahead.  The waves'
// sums meet in LDS, splits in a second launch, where the sink enters.
#include "window_common.h"

namespace slm {

typedef short wdr_v4 __attribute__((ext_vector_type(4)));
typedef short wdr_v8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) wdr_v4 wdr_lds_v4;

struct WindowDecodeK {
  slm_window_attn_args a;
  float* o_part;    // [rows, heads, splits, v_pad]
  float* ml_part;   // [rows, heads, splits, 2]
  int n_splits, head_blocks;
};

__device__ __forceinline__ float over_groups(float v, bool take_max) {
  const float x = __shfl_xor(v, 16, 64);
  v = take_max ? fmaxf(v, x) : v + x;
  const float y = __shfl_xor(v, 32, 64);
  return take_max ? fmaxf(v, y) : v + y;
}

template <int DQ, int VP>
__global__ void __launch_bounds__(256) window_decode_kernel(const WindowDecodeK p) {
  constexpr int KT = 32, QS = DQ / 32, NT = VP / 16;
  constexpr int VLS = VP * 2 + 16;                          // bytes of a value row in LDS
  constexpr int VCH = VP / 8, NV = KT * VCH / 64;
  constexpr int OS = VP + 4;                                // floats of an output row in LDS
  constexpr int WAVE_LDS = (KT * VLS > 16 * OS * 4 ? KT * VLS : 16 * OS * 4);
  __shared__ __attribute__((aligned(16))) char lds[4 * WAVE_LDS];
  __shared__ float sm[4][16], sl[4][16];
  const slm_window_attn_args& a = p.a;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l16 = lane & 15, g = lane >> 4;
  const int group = a.heads / a.kv_heads;
  int b = blockIdx.x;
  const int split = b % p.n_splits;
  b /= p.n_splits;
  const int hb = b % p.head_blocks;
  b /= p.head_blocks;
  const int kvh = b % a.kv_heads;
  const int64_t row = b / a.kv_heads;
  const int seq = seq_of_row(a.q_cu, a.batch, (int)row);
  const int32_t* table = a.block_table + a.block_cu[seq];
  const VisibleKeys vis(a.positions[row], a.window, a.keep_first);
  const int tiles = (vis.count + KT - 1) / KT, per = (tiles + p.n_splits - 1) / p.n_splits;
  const int t1 = min(tiles, (split + 1) * per);

  const int qh = kvh * group + min(16 * hb + l16, group - 1);
  bf16x8_t qf[QS];
  {
    const bf16* q = reinterpret_cast<const bf16*>(a.q) + row * a.ld_q + (int64_t)qh * DQ + 8 * g;
#pragma unroll
    for (int s = 0; s < QS; ++s) qf[s] = *reinterpret_cast<const bf16x8_t*>(q + 32 * s);
  }
  const bf16* kc = reinterpret_cast<const bf16*>(a.key_cache) + (int64_t)kvh * DQ + 8 * g;
  const bf16* vc = reinterpret_cast<const bf16*>(a.value_cache) + (int64_t)kvh * VP;
  const int64_t k_w = (int64_t)a.kv_heads * DQ, v_w = (int64_t)a.kv_heads * VP;
  char* v_lds = lds + wave * WAVE_LDS;

  auto slot_of = [&](int t) {   // of key lane % 32 of tile t (keys past the end: the last one, masked)
    const int pos = vis.position(min(t * KT + (lane & 31), vis.count - 1));
    return table[pos / a.block_size] + pos % a.block_size;
  };
  bf16x8_t kf[2][QS];
  u32x4 vf[NV];
  auto load_tile = [&](int slot) {
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const bf16* k = kc + (int64_t)__shfl(slot, 16 * n + l16, 64) * k_w;
#pragma unroll
      for (int s = 0; s < QS; ++s) kf[n][s] = *reinterpret_cast<const bf16x8_t*>(k + 32 * s);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int idx = lane + 64 * i;
      vf[i] = *reinterpret_cast<const u32x4*>(vc + (int64_t)__shfl(slot, idx / VCH, 64) * v_w + 8 * (idx % VCH));
    }
  };
  f32x4 o[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = M_INIT_F, l_run = 0.f;
  const bool capped = a.softcap > 0.f;
  const float scale2 = a.scale * LOG2E_F, cap2 = a.softcap * LOG2E_F, cap_in = capped ? 2.0f * LOG2E_F * a.scale / a.softcap : 0.f;
  // transpose read: key 4 g + l16 / 4, columns 4 (l16 % 4)
  const uint32_t tr_base = (uint32_t)(uintptr_t)v_lds + (uint32_t)((4 * g + (l16 >> 2)) * VLS + (l16 & 3) * 8);

  int t = split * per + wave;
  int slot = 0;
  if (t < t1) {
    load_tile(slot_of(t));
    slot = slot_of(min(t + 4, t1 - 1));
  }
  for (; t < t1; t += 4) {
    f32x4 s[2];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      s[n] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < QS; ++i) s[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[n][i], qf[i], s[n], 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int idx = lane + 64 * i;
      *reinterpret_cast<u32x4*>(v_lds + idx / VCH * VLS + idx % VCH * 16) = vf[i];
    }
    if (t + 4 < t1) {
      load_tile(slot);
      slot = slot_of(min(t + 8, t1 - 1));
    }
    // lane: head l16, keys 16 n + 4 g + e
    float mx = M_INIT_F;
#pragma unroll
    for (int n = 0; n < 2; ++n)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float x = capped ? cap2 * (1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + fast_exp2(s[n][e] * cap_in))) : s[n][e] * scale2;
        if (t * KT + 16 * n + 4 * g + e >= vis.count) x = -INFINITY;
        s[n][e] = x;
        mx = fmaxf(mx, x);
      }
    const float m_new = fmaxf(m_run, over_groups(mx, true));
    const float alpha = fast_exp2(m_run - m_new);
    m_run = m_new;
    float sum = 0.f;
    u32x4 w;
#pragma unroll
    for (int n = 0; n < 2; ++n)
#pragma unroll
      for (int e = 0; e < 4; e += 2) {
        const float e0 = fast_exp2(s[n][e] - m_new), e1 = fast_exp2(s[n][e + 1] - m_new);
        sum += e0 + e1;
        w[2 * n + (e >> 1)] = pack2<bf16_tag>(e0, e1);
      }
    l_run = l_run * alpha + sum;
    const bf16x8_t pf = __builtin_bit_cast(bf16x8_t, w);
    if (__any(alpha != 1.0f)) {
#pragma unroll
      for (int i = 0; i < NT; ++i) o[i] *= alpha;
    }
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");   // (the tile is the wave's own: order, no barrier)
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const uint32_t ad = tr_base + 32u * i;
      const wdr_v4 v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((wdr_lds_v4*)(uintptr_t)ad);
      const wdr_v4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((wdr_lds_v4*)(uintptr_t)(ad + 16 * VLS));
      const wdr_v8 v = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
      o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, v), pf, o[i], 0, 0, 0);
    }
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
  }
  l_run = over_groups(l_run, false);
  if (g == 0) sm[wave][l16] = m_run, sl[wave][l16] = l_run;
  float* ot = reinterpret_cast<float*>(v_lds);
#pragma unroll
  for (int i = 0; i < NT; ++i) *reinterpret_cast<f32x4*>(ot + l16 * OS + 16 * i + 4 * g) = o[i];
  __syncthreads();
  const int n_heads = min(16, group - 16 * hb);
  for (int i = tid; i < n_heads * (VP / 4); i += 256) {
    const int h = i / (VP / 4), c = i % (VP / 4) * 4, head = kvh * group + 16 * hb + h;
    float top = fmaxf(fmaxf(sm[0][h], sm[1][h]), fmaxf(sm[2][h], sm[3][h])), sink2 = 0.f;
    const bool whole = p.n_splits == 1;
    if (whole && a.sink) {
      sink2 = a.sink[head] * LOG2E_F;
      top = fmaxf(top, sink2);
    }
    float l = whole && a.sink ? fast_exp2(sink2 - top) : 0.f;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float f = fast_exp2(sm[w][h] - top);
      l = __builtin_fmaf(f, sl[w][h], l);
      v += *reinterpret_cast<const f32x4*>(reinterpret_cast<const float*>(lds + w * WAVE_LDS) + h * OS + c) * f;
    }
    if (whole) {
      v *= a.out_scale / l;
      *reinterpret_cast<u32x2*>(reinterpret_cast<bf16*>(a.out) + row * a.ld_out + (int64_t)head * VP + c) =
          u32x2{pack2<bf16_tag>(v.x, v.y), pack2<bf16_tag>(v.z, v.w)};
    } else {
      const int64_t pi = (row * a.heads + head) * p.n_splits + split;
      *reinterpret_cast<f32x4*>(p.o_part + pi * VP + c) = v;
      if (c == 0) p.ml_part[2 * pi] = top, p.ml_part[2 * pi + 1] = l;
    }
  }
}

__global__ void __launch_bounds__(256) window_combine_kernel(const WindowDecodeK p) {
  const slm_window_attn_args& a = p.a;
  const int c4 = a.v_pad / 4, n = p.n_splits;
  const int64_t quad = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (quad >= a.rows * a.heads * c4) return;
  const int64_t rh = quad / c4;
  const int c = (int)(quad % c4) * 4, head = (int)(rh % a.heads);
  const float* ml = p.ml_part + 2 * rh * n;
  const float* src = p.o_part + rh * n * a.v_pad + c;
  const float sink2 = a.sink ? a.sink[head] * LOG2E_F : M_INIT_F;
  float top = sink2;
  for (int s = 0; s < n; ++s) top = fmaxf(top, ml[2 * s]);
  float l = a.sink ? fast_exp2(sink2 - top) : 0.f;
  f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int s = 0; s < n; ++s) {
    const float f = fast_exp2(ml[2 * s] - top);
    l = __builtin_fmaf(f, ml[2 * s + 1], l);
    v += *reinterpret_cast<const f32x4*>(src + (int64_t)s * a.v_pad) * f;
  }
  v *= a.out_scale / l;
  *reinterpret_cast<u32x2*>(reinterpret_cast<bf16*>(a.out) + rh / a.heads * a.ld_out + (int64_t)head * a.v_pad + c) =
      u32x2{pack2<bf16_tag>(v.x, v.y), pack2<bf16_tag>(v.z, v.w)};
}

static int head_blocks(const slm_window_attn_args& a) { return (a.heads / a.kv_heads + 15) / 16; }
// splits: about four workgroups per CU, at least 128 keys (a tile per wave) each
static int split_count(const slm_window_attn_args& a) {
  if (a.n_splits > 0) return a.n_splits < 64 ? a.n_splits : 64;
  int64_t keys = a.max_kv_len;
  if (a.window > 0 && keys > (int64_t)a.window + (a.keep_first > 0 ? a.keep_first : 0)) keys = (int64_t)a.window + (a.keep_first > 0 ? a.keep_first : 0);
  const int64_t wgs = a.rows * a.kv_heads * head_blocks(a);
  const int64_t want = (1024 + wgs - 1) / wgs, most = keys / 128;
  const int64_t n = want < most ? want : most;
  return (int)(n < 1 ? 1 : n > 64 ? 64 : n);
}

static bool wd_width(int w) { return w == 64 || w == 96 || w == 128 || w == 192 || w == 256; }
bool window_decode_ok(const slm_window_attn_args& a) {
  return a.dtype == SLM_BF16 && wd_width(a.d_pad) && wd_width(a.v_pad) && a.rows * a.kv_heads * head_blocks(a) * 64 < 0x7fffffff;
}
size_t window_decode_workspace(const slm_window_attn_args& a) {
  const int n = split_count(a);
  return n == 1 ? 0 : (size_t)a.rows * a.heads * n * (a.v_pad + 2) * 4;
}

template <int DQ, int VP>
static void wd_launch(const WindowDecodeK& p, hipStream_t st) {
  const int64_t grid = p.a.rows * p.a.kv_heads * p.head_blocks * p.n_splits;
  window_decode_kernel<DQ, VP><<<dim3((unsigned)grid), dim3(256), 0, st>>>(p);
}
template <int DQ>
static void wd_v(const WindowDecodeK& p, hipStream_t st) {
  switch (p.a.v_pad) {
    case 64: wd_launch<DQ, 64>(p, st); break;
    case 96: wd_launch<DQ, 96>(p, st); break;
    case 128: wd_launch<DQ, 128>(p, st); break;
    case 192: wd_launch<DQ, 192>(p, st); break;
    default: wd_launch<DQ, 256>(p, st);
  }
}
int window_decode(const slm_window_attn_args& a, hipStream_t st) {
  WindowDecodeK p;
  p.a = a;
  p.n_splits = split_count(a);
  p.head_blocks = head_blocks(a);
  p.o_part = p.ml_part = nullptr;
  if (p.n_splits > 1) {
    if (!a.workspace || a.workspace_bytes < window_decode_workspace(a)) return SLM_ERR_WORKSPACE;
    if (!aligned16(a.workspace)) return SLM_ERR_ALIGNMENT;
    p.o_part = reinterpret_cast<float*>(a.workspace);
    p.ml_part = p.o_part + a.rows * a.heads * p.n_splits * a.v_pad;
  }
  hip_clear_error();
  switch (a.d_pad) {
    case 64: wd_v<64>(p, st); break;
    case 96: wd_v<96>(p, st); break;
    case 128: wd_v<128>(p, st); break;
    case 192: wd_v<192>(p, st); break;
    default: wd_v<256>(p, st);
  }
  int rc = hip_check_launch();
  if (rc != SLM_OK || p.n_splits == 1) return rc;
  const int64_t quads = a.rows * a.heads * (a.v_pad / 4);
  window_combine_kernel<<<dim3((unsigned)((quads + 255) / 256)), dim3(256), 0, st>>>(p);
  return hip_check_launch();
}

}  // namespace slm
