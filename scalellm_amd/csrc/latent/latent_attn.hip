// latent_attn.hip -- attention of single query rows over the paged latent cache ("absorbed" form: the
// unrotated query is already multiplied by W_uk, so every head scores against the cached row itself and
// accumulates the cached latent; W_uv is applied to the result).  All heads share every cache byte.
//
// Work item: (query row, block of 16 MH heads, split of its visible range).  Visible = positions
// [max(0, p - window + 1), p] of the row's sequence; a portion of several tokens is several rows.
//
// latent_attn_kernel (bf16, MFMA 16x16x32), four waves, KT cache rows per tile:
//   staging   global -> registers (the next tile, in flight across the whole tile) -> LDS, rows padded to an odd
//             number of 16-byte units so that both fragment reads below are bank-conflict free
//   S = C Q^T each wave one 16 x 16 block or two (A = cache rows, B = its head block, held in registers), S to LDS
//   softmax   every wave reads the scores back in the B layout of the second product (column = head = lane % 16,
//             8 consecutive keys) and does the row statistics itself: no second exchange, one scalar per lane
//   O^T += C^T P^T   wave w owns a quarter of the latent columns; A = C^T out of the row-major tile by the transpose
//             read (ds_read_b64_tr_b16: 4 keys of one column per lane)
// Bound: HBM (the cache stream) for 16 heads; the score exchange and the redundant soft-max are what a wide
// head block costs.
//
// latent_attn_any_kernel: any size, any dtype, VALU: the 32-bit path and sizes without an MFMA form.
#include "latent_common.h"

namespace slm {

constexpr int LA_MAX_SPLITS = 64;

struct LatentAttnK {
  slm_latent_attn_args a;
  int n_splits;
  float* o_part;   // [rows][heads][n_splits][c_pad]
  float* ml_part;  // [rows][heads][n_splits][2]
  float scale2;    // scale * log2(e)
  int block_shift, block_mask;
};

typedef short tr_v4 __attribute__((ext_vector_type(4)));
typedef short tr_v8 __attribute__((ext_vector_type(8)));
typedef __attribute__((address_space(3))) tr_v4 tr_lds_v4;

template <int KP, int RP, int MH>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2)))
latent_attn_kernel(const LatentAttnK p) {
  constexpr int R = KP + RP;
  constexpr int KT = MH == 1 ? 64 : 32;      // cache rows per tile
  constexpr int CH = R / 8;                  // 16-byte chunks of a row
  constexpr int LS = R * 2 + 16;             // LDS row stride (bytes): an odd number of 16-byte units
  constexpr int NCH = (KT * CH + 255) / 256; // chunks per thread and tile
  constexpr int QS = R / 32;                 // MFMA k-steps of the scores
  constexpr int KS = KT / 32;                // MFMA k-steps of the second product
  constexpr int NT = KP / 64;                // 16-column blocks of the latent per wave
  constexpr int SS = KT + 4;                 // score row stride (floats)
  constexpr int UK = (KT / 16) * MH / 4;     // score blocks per wave (same head block, key blocks 4 / MH apart)
  static_assert(UK >= 1 && (KT / 16) * MH % 4 == 0, "score blocks per wave");
  __shared__ __attribute__((aligned(16))) char tile[KT * LS];
  __shared__ __attribute__((aligned(16))) float sc[16 * MH * SS];
  __shared__ int slot_lds[2][KT];

  const slm_latent_attn_args& a = p.a;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l16 = lane & 15, g = lane >> 4;
  const int hblocks = (a.heads + 16 * MH - 1) / (16 * MH);
  // head blocks of one (row, split) sit 8 blocks apart in the grid: they share a cache range and, dispatched
  // round-robin over the 8 XCDs, an L2
  const int64_t items = a.rows * p.n_splits;
  const int64_t group = blockIdx.x / (8 * hblocks), in_group = blockIdx.x % (8 * hblocks);
  const int64_t item = group * 8 + in_group % 8;
  const int hb = (int)(in_group / 8);
  if (item >= items) return;
  const int64_t row = item / p.n_splits;
  const int split = (int)(item % p.n_splits);
  const int h0 = hb * 16 * MH;

  const int seq = seq_of_row(a.q_cu, a.batch, (int)row);
  const int pos = a.positions[row];
  const int bcu = a.block_cu[seq];
  int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  int hi = pos + 1;
  if (p.n_splits > 1) {
    const int tiles = (hi - lo + KT - 1) / KT;
    const int per = (tiles + p.n_splits - 1) / p.n_splits * KT;
    lo = min(hi, lo + split * per);
    hi = min(hi, lo + per);
  }
  const int n_tiles = (hi - lo + KT - 1) / KT;

  const char* cache = reinterpret_cast<const char*>(a.cache);
  auto slot_of = [&](int key) {
    key = min(key, hi - 1);  // rows past the end re-read the last one; masked below
    return a.block_table[bcu + (key >> p.block_shift)] + (key & p.block_mask);
  };

  u32x4 stage[NCH];
  auto load_tile = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      const int idx = tid + 256 * i;
      const int r = idx / CH, c = idx % CH;
      if ((KT * CH) % 256 == 0 || idx < KT * CH)
        stage[i] = *reinterpret_cast<const u32x4*>(cache + (int64_t)slot_lds[buf][r] * (R * 2) + 16 * c);
    }
  };
  auto store_tile = [&]() {
#pragma unroll
    for (int i = 0; i < NCH; ++i) {
      const int idx = tid + 256 * i;
      const int r = idx / CH, c = idx % CH;
      if ((KT * CH) % 256 == 0 || idx < KT * CH) *reinterpret_cast<u32x4*>(tile + r * LS + 16 * c) = stage[i];
    }
  };

  // this wave's head block of the scores, as B fragments
  const int hw = wave % MH;
  bf16x8_t qf[QS];
  {
    const int h = h0 + 16 * hw + l16;
    const bf16* q = reinterpret_cast<const bf16*>(a.q_abs) + (row * a.heads + min(h, a.heads - 1)) * R + 8 * g;
#pragma unroll
    for (int s = 0; s < QS; ++s) qf[s] = *reinterpret_cast<const bf16x8_t*>(q + 32 * s);
  }
  f32x4 o[MH][NT];
  float m_run[MH], l_run[MH];
#pragma unroll
  for (int m = 0; m < MH; ++m) {
    m_run[m] = M_INIT_F;
    l_run[m] = 0.f;
#pragma unroll
    for (int t = 0; t < NT; ++t) o[m][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  if (n_tiles > 0) {
    if (tid < KT) {
      slot_lds[0][tid] = slot_of(lo + tid);
      slot_lds[1][tid] = slot_of(lo + KT + tid);
    }
    lds_barrier();
    load_tile(0);
  }
  // transpose-read address of this lane: keys 8 g + (lane % 16) / 4 (+ 4 for the second half), column chunk lane % 4
  const uint32_t tr_base = (uint32_t)(uintptr_t)tile + (uint32_t)((8 * g + (l16 >> 2)) * LS + (l16 & 3) * 8 + wave * (KP / 4) * 2);

  for (int t = 0; t < n_tiles; ++t) {
    const int k0 = lo + t * KT;
    store_tile();
    lds_barrier();
    if (t + 1 < n_tiles) load_tile((t + 1) & 1);
    // ---- scores
#pragma unroll
    for (int u = 0; u < UK; ++u) {
      const int kb = wave / MH + u * (4 / MH);
      const char* kp = tile + (16 * kb + l16) * LS + 16 * g;
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < QS; ++i)
        s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(kp + 64 * i), qf[i], s, 0, 0, 0);
      // lane: head l16, keys 16 kb + 4 g .. + 3
      *reinterpret_cast<f32x4*>(&sc[(16 * hw + l16) * SS + 16 * kb + 4 * g]) = s;
    }
    lds_barrier();
    if (tid < KT && t + 2 < n_tiles) slot_lds[t & 1][tid] = slot_of(k0 + 2 * KT + tid);
    // ---- soft-max, in the B layout of the second product
    bf16x8_t pf[MH][KS];
#pragma unroll
    for (int m = 0; m < MH; ++m) {
      float v[KS][8];
      float mx = M_INIT_F;
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const float* sp = &sc[(16 * m + l16) * SS + 32 * k + 8 * g];
        const f32x4 x = *reinterpret_cast<const f32x4*>(sp), y = *reinterpret_cast<const f32x4*>(sp + 4);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float raw = j < 4 ? x[j & 3] : y[j & 3];
          v[k][j] = k0 + 32 * k + 8 * g + j < hi ? raw * p.scale2 : -INFINITY;
          mx = fmaxf(mx, v[k][j]);
        }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float m_new = fmaxf(m_run[m], mx);
      const float alpha = fast_exp2(m_run[m] - m_new);
      m_run[m] = m_new;
      float sum = 0.f;
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        u32x4 w;
#pragma unroll
        for (int j = 0; j < 8; j += 2) {
          const float e0 = fast_exp2(v[k][j] - m_new), e1 = fast_exp2(v[k][j + 1] - m_new);
          sum += e0 + e1;
          w[j >> 1] = pack2<bf16_tag>(e0, e1);
        }
        pf[m][k] = __builtin_bit_cast(bf16x8_t, w);
      }
      l_run[m] = l_run[m] * alpha + sum;
      if (__any(alpha != 1.0f)) {
#pragma unroll
        for (int t2 = 0; t2 < NT; ++t2) o[m][t2] *= alpha;
      }
    }
    // ---- O^T += C^T P^T
#pragma unroll
    for (int t2 = 0; t2 < NT; ++t2)
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const uint32_t ad = tr_base + (uint32_t)(32 * k * LS + 32 * t2);
        const tr_v4 c0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((tr_lds_v4*)ad);
        const tr_v4 c1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((tr_lds_v4*)(ad + 4 * LS));
        const tr_v8 c = __builtin_shufflevector(c0, c1, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
        for (int m = 0; m < MH; ++m)
          o[m][t2] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, c), pf[m][k], o[m][t2], 0, 0, 0);
      }
    lds_barrier();
  }

  // lane: head l16 of block m, latent columns wave * KP / 4 + 16 t + 4 g .. + 3
#pragma unroll
  for (int m = 0; m < MH; ++m) {
    float l = l_run[m];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    const int h = h0 + 16 * m + l16;
    if (h >= a.heads) continue;
    const int64_t rh = row * a.heads + h;
    const int c0 = wave * (KP / 4) + 4 * g;
    if (p.n_splits == 1) {
      const float inv = 1.0f / l;  // (every row sees itself: l > 0)
      bf16* out = reinterpret_cast<bf16*>(a.out) + rh * KP + c0;
#pragma unroll
      for (int t = 0; t < NT; ++t)
        *reinterpret_cast<u32x2*>(out + 16 * t) = u32x2{pack2<bf16_tag>(o[m][t].x * inv, o[m][t].y * inv),
                                                        pack2<bf16_tag>(o[m][t].z * inv, o[m][t].w * inv)};
    } else {
      const int64_t pi = rh * p.n_splits + split;
      float* out = p.o_part + pi * KP + c0;
#pragma unroll
      for (int t = 0; t < NT; ++t) *reinterpret_cast<f32x4*>(out + 16 * t) = o[m][t];
      if (wave == 0 && g == 0) {
        p.ml_part[2 * pi] = m_run[m];
        p.ml_part[2 * pi + 1] = l;
      }
    }
  }
}

// merges the splits of one (row, head): c_pad / 4 threads' worth of columns, 4 per thread
__global__ void __launch_bounds__(128) latent_attn_combine_kernel(const LatentAttnK p) {
  const int64_t rh = blockIdx.x;
  const int c_pad = p.a.c_pad, n = p.n_splits;
  const float* ml = p.ml_part + 2 * rh * n;
  float m = M_INIT_F;
  for (int s = 0; s < n; ++s) m = fmaxf(m, ml[2 * s]);
  float l = 0.f;
  for (int s = 0; s < n; ++s) l += ml[2 * s + 1] * fast_exp2(ml[2 * s] - m);
  const float inv = 1.0f / l;
  for (int c = 4 * threadIdx.x; c < c_pad; c += 512) {
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < n; ++s) {
      const float w = fast_exp2(ml[2 * s] - m);
      o += *reinterpret_cast<const f32x4*>(p.o_part + (rh * n + s) * c_pad + c) * w;
    }
    *reinterpret_cast<u32x2*>(reinterpret_cast<bf16*>(p.a.out) + rh * c_pad + c) =
        u32x2{pack2<bf16_tag>(o.x * inv, o.y * inv), pack2<bf16_tag>(o.z * inv, o.w * inv)};
  }
}

constexpr int ANY_COLS = 8;  // latent columns per thread (c_pad <= 2048)

template <typename E>
__global__ void __launch_bounds__(256) latent_attn_any_kernel(const LatentAttnK p) {
  extern __shared__ float q_lds[];  // the absorbed query
  __shared__ float pr[256];
  __shared__ int slots[256];
  __shared__ float red[4];
  const slm_latent_attn_args& a = p.a;
  const int tid = threadIdx.x, R = a.c_pad + a.r_pad;
  const int64_t row = blockIdx.x / a.heads, rh = blockIdx.x;
  const int seq = seq_of_row(a.q_cu, a.batch, (int)row);
  const int pos = a.positions[row], bcu = a.block_cu[seq];
  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0, hi = pos + 1;
  const E* cache = reinterpret_cast<const E*>(a.cache);
  for (int i = tid; i < R; i += 256) q_lds[i] = to_f32(reinterpret_cast<const E*>(a.q_abs)[rh * R + i]);
  float acc[ANY_COLS];
#pragma unroll
  for (int c = 0; c < ANY_COLS; ++c) acc[c] = 0.f;
  float m = M_INIT_F, l = 0.f;
  for (int k0 = lo; k0 < hi; k0 += 256) {
    __syncthreads();
    const int key = k0 + tid;
    float s = -INFINITY;
    if (key < hi) {
      const int slot = a.block_table[bcu + (key >> p.block_shift)] + (key & p.block_mask);
      slots[tid] = slot;
      const E* r = cache + (int64_t)slot * R;
      float d = 0.f;
      for (int i = 0; i < R; i += 4) {
        float v[4];
        load_f32<4>(r + i, v);
#pragma unroll
        for (int j = 0; j < 4; ++j) d = __builtin_fmaf(v[j], q_lds[i + j], d);
      }
      s = d * a.scale;
    }
    const float m_new = fmaxf(m, block_max256(s, red));
    const float e = key < hi ? expf(s - m_new) : 0.f;
    const float alpha = expf(m - m_new);
    pr[tid] = e;
    l = l * alpha + block_sum256(e, red);
    m = m_new;
    __syncthreads();
    const int n = min(256, hi - k0);
#pragma unroll
    for (int c = 0; c < ANY_COLS; ++c) {
      const int col = tid + 256 * c;
      if (col < a.c_pad) {
        float v = acc[c] * alpha;
        for (int j = 0; j < n; ++j) v = __builtin_fmaf(pr[j], to_f32(cache[(int64_t)slots[j] * R + col]), v);
        acc[c] = v;
      }
    }
  }
#pragma unroll
  for (int c = 0; c < ANY_COLS; ++c) {
    const int col = tid + 256 * c;
    if (col < a.c_pad) reinterpret_cast<E*>(a.out)[rh * a.c_pad + col] = (E)(acc[c] / l);
  }
}

static int la_mh(int heads) { return heads > 32 ? 4 : heads > 16 ? 2 : 1; }
static bool la_mfma(int c_pad, int r_pad, int dtype) {
  return dtype == SLM_BF16 && (c_pad == 64 || c_pad == 128 || c_pad == 256 || c_pad == 512) && (r_pad == 32 || r_pad == 64);
}
static int la_splits(const slm_latent_attn_args& a) {
  if (!la_mfma(a.c_pad, a.r_pad, a.dtype) || a.generic) return 1;
  if (a.n_splits > 0) return a.n_splits < LA_MAX_SPLITS ? a.n_splits : LA_MAX_SPLITS;
  const int mh = la_mh(a.heads), kt = mh == 1 ? 64 : 32;
  const int64_t wgs = a.rows * ((a.heads + 16 * mh - 1) / (16 * mh));
  int64_t len = a.max_kv_len > 0 ? a.max_kv_len : 1;
  if (a.window > 0 && a.window < len) len = a.window;
  const int64_t tiles = (len + kt - 1) / kt;
  int64_t n = 512 / (wgs > 0 ? wgs : 1);        // two workgroups per CU
  const int64_t cap = (tiles + 1) / 2;            // at least two tiles each
  if (n > cap) n = cap;
  if (n > LA_MAX_SPLITS) n = LA_MAX_SPLITS;
  return n < 1 ? 1 : (int)n;
}

template <int KP, int RP, int MH>
static void la_launch(const LatentAttnK& p, hipStream_t st) {
  const int hblocks = (p.a.heads + 16 * MH - 1) / (16 * MH);
  const int64_t groups = (p.a.rows * p.n_splits + 7) / 8;
  latent_attn_kernel<KP, RP, MH><<<dim3((unsigned)(groups * 8 * hblocks)), dim3(256), 0, st>>>(p);
}
template <int KP, int RP>
static void la_heads(const LatentAttnK& p, hipStream_t st) {
  switch (la_mh(p.a.heads)) {
    case 1: la_launch<KP, RP, 1>(p, st); break;
    case 2: la_launch<KP, RP, 2>(p, st); break;
    default: la_launch<KP, RP, 4>(p, st);
  }
}
template <int KP>
static void la_rot(const LatentAttnK& p, hipStream_t st) {
  if (p.a.r_pad == 32) la_heads<KP, 32>(p, st);
  else la_heads<KP, 64>(p, st);
}

static int la_check(const slm_latent_attn_args* a) {
  if (!a || a->rows < 0 || a->batch < 1 || a->heads < 1 || a->c_pad < 64 || a->c_pad % 64 || a->r_pad < 32 || a->r_pad % 32 ||
      !is_pow2(a->block_size))
    return SLM_ERR_INVALID_ARG;
  if (a->dtype != SLM_BF16 && a->dtype != SLM_F32) return SLM_ERR_UNSUPPORTED;
  if (a->c_pad > 256 * ANY_COLS || a->r_pad > 1024) return SLM_ERR_UNSUPPORTED;
  return SLM_OK;
}

}  // namespace slm

using namespace slm;

extern "C" SLM_API int slm_latent_attn_is_mfma(int32_t c_pad, int32_t r_pad, int32_t dtype) {
  return la_mfma(c_pad, r_pad, dtype) ? 1 : 0;
}
extern "C" SLM_API size_t slm_latent_attn_workspace_bytes(const slm_latent_attn_args* a) {
  if (la_check(a) != SLM_OK) return 0;
  const int n = la_splits(*a);
  return n <= 1 ? 0 : (size_t)a->rows * a->heads * n * (a->c_pad + 2) * 4;
}
extern "C" SLM_API int slm_latent_attn(const slm_latent_attn_args* a, void* stream) {
  const int rc = la_check(a);
  if (rc != SLM_OK) return rc;
  if (!a->q_abs || !a->cache || !a->out || !a->positions || !a->q_cu || !a->block_table || !a->block_cu) return SLM_ERR_INVALID_ARG;
  if (!aligned16(a->q_abs) || !aligned16(a->cache) || !aligned16(a->out)) return SLM_ERR_ALIGNMENT;
  if (a->rows == 0) return SLM_OK;
  LatentAttnK p;
  p.a = *a;
  p.n_splits = la_splits(*a);
  p.scale2 = a->scale * LOG2E_F;
  p.block_shift = ilog2(a->block_size);
  p.block_mask = a->block_size - 1;
  p.o_part = p.ml_part = nullptr;
  if (p.n_splits > 1) {
    if (!a->workspace || !aligned16(a->workspace) || a->workspace_bytes < slm_latent_attn_workspace_bytes(a)) return SLM_ERR_WORKSPACE;
    p.o_part = (float*)a->workspace;
    p.ml_part = p.o_part + (size_t)a->rows * a->heads * p.n_splits * a->c_pad;
  }
  hipStream_t st = (hipStream_t)stream;
  hip_clear_error();
  if (!a->generic && la_mfma(a->c_pad, a->r_pad, a->dtype)) {
    switch (a->c_pad) {
      case 64: la_rot<64>(p, st); break;
      case 128: la_rot<128>(p, st); break;
      case 256: la_rot<256>(p, st); break;
      default: la_rot<512>(p, st);
    }
    if (p.n_splits > 1) latent_attn_combine_kernel<<<dim3((unsigned)(a->rows * a->heads)), dim3(128), 0, st>>>(p);
  } else {
    const dim3 grid((unsigned)(a->rows * a->heads));
    const size_t lds = (size_t)(a->c_pad + a->r_pad) * 4;
    if (a->dtype == SLM_BF16) latent_attn_any_kernel<bf16><<<grid, dim3(256), lds, st>>>(p);
    else latent_attn_any_kernel<float><<<grid, dim3(256), lds, st>>>(p);
  }
  return hip_check_launch();
}
