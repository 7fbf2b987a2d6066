// latent_attn.hip -- attention of single query rows over the paged latent cache ("absorbed" form: the
// unrotated query is already multiplied by W_uk, so every head scores against the cached row itself and
// accumulates the cached latent; W_uv is applied to the result).  All heads share every cache byte.
//
// Work item: (query row, block of 16 MH heads, split of its visible range).  Visible = positions
// [max(0, p - window + 1), p] of the row's sequence; a portion of several tokens is several rows.
//
// latent_attn_kernel (bf16, MFMA 16x16x32), eight waves, 32 cache rows per tile, a ring of four to eight tiles in LDS:
//   staging   global -> LDS by LDS-DMA (a wave instruction writes 1 KiB linearly), all but one tile of the ring in flight
//             behind counted waits; block-table entries of the range are staged in LDS first (LA_TBL at a time), so
//             no other load sits in the vmcnt queue.  The image is swizzled on the source side: 16-byte unit u of row r holds chunk
//             u ^ (r / 2 % 8), which keeps both fragment reads below off each other's banks
//   S = C Q^T 16 x 16 blocks, one a wave (16 heads: half a contraction each), A = cache rows, B = the wave's head
//             block, held in registers; S to LDS.  One tile AHEAD of the rest, so that a tile costs one barrier and a
//             wave's soft-max has another tile's products to hide behind
//   softmax   every wave reads the scores back in the B layout of the second product (column = head = lane % 16,
//             8 consecutive keys) and does the row statistics itself: no second exchange, one scalar per lane
//   O^T += C^T P^T   wave w owns an eighth of the latent columns; A = C^T out of the row-major tile by the transpose
//             read (ds_read_b64_tr_b16: 4 keys of one column per lane)
// Bound: HBM (the cache stream) for 16 heads; the score exchange and the redundant soft-max are what a wide
// head block costs.  Ranges that are split leave fp32 partials for latent_attn_combine_kernel.
//
// latent_attn_any_kernel: any size, any dtype, VALU: the 32-bit path and sizes without an MFMA form.
#include "latent_common.h"

namespace slm {

constexpr int LA_MAX_SPLITS = 128;

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

// maximum over the four lanes that share lane % 16
__device__ __forceinline__ float max_over_groups(float x) {
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  x = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}

// waits until at most `tiles` tiles of PER DMA instructions each are in flight (0 <= tiles <= MAX)
template <int MAX, int PER>
__device__ __forceinline__ void wait_tiles(int tiles) {
  if constexpr (MAX > 0) {
    if (tiles < MAX) return wait_tiles<MAX - 1, PER>(tiles);
  }
  asm volatile("s_waitcnt vmcnt(%0)" : : "n"(MAX * PER) : "memory");
}

constexpr int LA_KT = 32;     // cache rows per tile
constexpr int LA_TBL = 1024;  // block-table entries staged in LDS at a time

template <int KP, int RP, int MH>
__global__ void __launch_bounds__(512) latent_attn_kernel(const LatentAttnK p) {
  constexpr int R = KP + RP;
  constexpr int KT = LA_KT;
  constexpr int CH = R / 8;                  // 16-byte chunks of a cache row
  constexpr int CHP = (CH + 7) / 8 * 8;      // 16-byte units of a row in LDS
  constexpr int ROWB = CHP * 16, TILE = KT * ROWB;
  constexpr int NTOT = KT * CHP / 64;        // DMA instructions of a tile: NHI in the first NTOT % 8 waves, NLO in the others
  constexpr int NHI = (NTOT + 7) / 8, NLO = NTOT / 8;
  constexpr int QS = R / 32;                 // MFMA k-steps of the scores
  constexpr int KH = MH == 1 ? 2 : 1;        // waves that share a score block's contraction
  constexpr int QW = (QS + KH - 1) / KH;     // k-steps per wave
  constexpr int NT = KP >= 128 ? KP / 128 : 1;  // 16-column blocks of the latent per wave
  constexpr int SS = KT + 4;                 // score row stride (floats)
  constexpr int SC = KH * 16 * MH * SS;      // floats of one tile's scores
  constexpr int FIT = (163840 - 8 * SC - 4 * LA_TBL) / TILE, NBUF = FIT > 8 ? 8 : FIT;  // tiles in the ring
  static_assert(NBUF >= 4 && (NBUF - 3) * NHI < 63, "ring and counted waits");
  __shared__ __attribute__((aligned(16))) char ring[NBUF * TILE];
  __shared__ __attribute__((aligned(16))) float sc[2][SC];
  __shared__ int tbl[LA_TBL];

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

  // score block of this wave: head block hw, key block kb, k-steps from kh * QW
  const int kb = wave & 1, hw = (wave >> 1) & (MH - 1), kh = KH == 2 ? (wave >> 1) & 1 : 0;
  const bool scorer = wave < 2 * MH * KH;
  bf16x8_t qf[QW];
  {
    const int h = h0 + 16 * hw + l16;
    const bf16* q = reinterpret_cast<const bf16*>(a.q_abs) + (row * a.heads + min(h, a.heads - 1)) * R + 8 * g;
#pragma unroll
    for (int s = 0; s < QW; ++s) {
      const int step = kh * QW + s;
      qf[s] = *reinterpret_cast<const bf16x8_t*>(q + 32 * min(step, QS - 1));
      if (KH * QW != QS && step >= QS) qf[s] = __builtin_bit_cast(bf16x8_t, u32x4{0u, 0u, 0u, 0u});
    }
  }

  // decode batches: row r is sequence r.  Looked up as if, all loads at once; otherwise the search
  const int guess = min((int)row, a.batch - 1);
  const int g0 = a.q_cu[guess], g1 = a.q_cu[guess + 1], pos = a.positions[row];
  int bcu = a.block_cu[guess];
  if (g0 != (int)row || g1 != (int)row + 1) bcu = a.block_cu[seq_of_row(a.q_cu, a.batch, (int)row)];
  int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  int hi = pos + 1;
  if (p.n_splits > 1) {
    const int tiles = (hi - lo + KT - 1) / KT;
    const int per = (tiles + p.n_splits - 1) / p.n_splits * KT;
    lo = min(hi, lo + split * per);
    hi = min(hi, lo + per);
  }
  // (the queries have arrived before the first DMA is issued: a wait for them later would drain the ring)
#pragma unroll
  for (int s = 0; s < QW; ++s) asm volatile("" : "+v"(qf[s]));

  // the segment of the range whose block-table entries are staged: keys [lo, hi)
  const int range_hi = hi;
  int blk0 = 0, n_tiles = 0;
  const uint32_t ring0 = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) char*)ring;
  const char* cache = reinterpret_cast<const char*>(a.cache);
  // (inline asm: through the builtin the compiler makes every read of the ring wait for the DMA into its other tiles)
  auto issue = [&](int t) {
    const uint32_t dst0 = ring0 + (uint32_t)(t % NBUF) * TILE;
    const char* src[NHI];
#pragma unroll
    for (int i = 0; i < NHI; ++i) {
      const int u = min(wave + 8 * i, NTOT - 1) * 64 + lane;
      const int r = u / CHP, c = min((u % CHP) ^ ((r >> 1) & 7), CH - 1);
      const int key = min(lo + t * KT + r, hi - 1);  // rows past the end re-read the last one; masked below
      const int slot = tbl[(key >> p.block_shift) - blk0];
      src[i] = cache + (int64_t)(slot + (key & p.block_mask)) * (R * 2) + 16 * c;
    }
#pragma unroll
    for (int i = 0; i < NHI; ++i)
      if (i < NLO || wave < NTOT % 8)
        asm volatile("s_mov_b32 m0, %1\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, off"
                     :
                     : "v"(src[i]), "s"(dst0 + (uint32_t)(wave + 8 * i) * 1024u)
                     : "memory", "m0");
  };

  f32x4 o[MH][NT];
  float m_run[MH], l_run[MH];
#pragma unroll
  for (int m = 0; m < MH; ++m) {
    m_run[m] = M_INIT_F;
    l_run[m] = 0.f;
#pragma unroll
    for (int t = 0; t < NT; ++t) o[m][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  // fragment reads: A of the scores (row l16 of a 16-key block, chunk 4 i + g), and the transpose read (keys
  // 8 g + l16 / 4 and + 4, 8-byte piece l16 % 4 of a 16-column block)
  const uint32_t k_row = (uint32_t)l16 * ROWB, k_x = (uint32_t)((l16 >> 1) & 7) ^ (uint32_t)g;
  const uint32_t tr_row = (uint32_t)(8 * g + (l16 >> 2)) * ROWB + (uint32_t)(l16 & 1) * 8u;
  const uint32_t tr_x0 = (uint32_t)((4 * g + (l16 >> 3)) & 7) ^ (uint32_t)((l16 >> 1) & 1);
  const uint32_t tr_x1 = (uint32_t)((4 * g + 2 + (l16 >> 3)) & 7) ^ (uint32_t)((l16 >> 1) & 1);
  const uint32_t tr_c = (uint32_t)wave * (2 * NT);
  const bool columns = KP >= 128 || wave < KP / 16;

  constexpr int QC = QW > 10 ? (QW + 1) / 2 : QW;   // k-steps read ahead of the products (register budget)
  bf16x8_t kf[QC];
  auto read_rows = [&](int t, int first) {   // A fragments of tile t, k-steps from `first` of this wave's
    const uint32_t base = ring0 + (uint32_t)(t % NBUF) * TILE + (uint32_t)(16 * kb) * ROWB + k_row;
#pragma unroll
    for (int i = 0; i < QC; ++i) {
      const uint32_t step = (uint32_t)(kh * QW + first + i);
      kf[i] = *(__attribute__((address_space(3))) const bf16x8_t*)(uintptr_t)(base + (((4u * min(step, (uint32_t)QS - 1)) ^ k_x) << 4));
    }
  };
  auto score = [&](int t) {
    f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < QW; c += QC) {
      if (c > 0) read_rows(t, c);
#pragma unroll
      for (int i = 0; i < QC; i += 2) {
        if (c + i < QW) s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i], qf[c + i], s0, 0, 0, 0);
        if (i + 1 < QC && c + i + 1 < QW) s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i + 1], qf[c + i + 1], s1, 0, 0, 0);
      }
    }
    // lane: head l16, keys 16 kb + 4 g .. + 3
    *reinterpret_cast<f32x4*>(&sc[t & 1][(16 * (MH * kh + hw) + l16) * SS + 16 * kb + 4 * g]) = s0 + s1;
  };
  auto arrived = [&](int younger) {   // the wave's part of a tile, with the younger tiles of the ring still in flight
    if (NTOT % 8 == 0 || wave < NTOT % 8) wait_tiles<NBUF - 2, NHI>(younger);
    else wait_tiles<NBUF - 2, NLO>(younger);
  };
  for (; lo < range_hi; lo = hi) {
    blk0 = lo >> p.block_shift;
    hi = min(range_hi, (blk0 + LA_TBL) << p.block_shift);
    n_tiles = (hi - lo + KT - 1) / KT;
    for (int i = tid; i <= ((hi - 1) >> p.block_shift) - blk0; i += 512) tbl[i] = a.block_table[bcu + blk0 + i];
    __syncthreads();
#pragma unroll 1
    for (int t = 0; t < min(NBUF - 1, n_tiles); ++t) issue(t);
    arrived(min(NBUF - 2, n_tiles - 1));
    lds_barrier();
    if (scorer) {
      read_rows(0, 0);
      score(0);
    }
    for (int t = 0; t < n_tiles; ++t) {
      const int k0 = lo + t * KT;
      if (t + 1 < n_tiles) arrived(min(NBUF - 3, n_tiles - 2 - t));
      lds_barrier();   // tile t + 1 and the scores of tile t are there, tile t - 1 is done with
      if (t + NBUF - 1 < n_tiles) issue(t + NBUF - 1);
      const uint32_t tile = ring0 + (uint32_t)(t % NBUF) * TILE;
      const bool next = scorer && t + 1 < n_tiles;
      if (next) read_rows(t + 1, 0);
      if (!columns) {   // (a latent of 64: four waves hold all of it)
        if (next) score(t + 1);
        continue;
      }
      // ---- scores back in the B layout of the second product, C^T fragments behind them (read under the soft-max)
      f32x4 raw[MH][KH][2];
#pragma unroll
      for (int m = 0; m < MH; ++m)
#pragma unroll
        for (int k = 0; k < KH; ++k) {
          const float* sp = &sc[t & 1][(16 * (MH * k + m) + l16) * SS + 8 * g];
          raw[m][k][0] = *reinterpret_cast<const f32x4*>(sp);
          raw[m][k][1] = *reinterpret_cast<const f32x4*>(sp + 4);
        }
      __builtin_amdgcn_sched_barrier(0);
      tr_v8 ct[NT];
#pragma unroll
      for (int t2 = 0; t2 < NT; ++t2) {
        const uint32_t cc = tr_c + 2u * t2, ad = tile + tr_row;
        const tr_v4 c0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((tr_lds_v4*)(uintptr_t)(ad + ((cc ^ tr_x0) << 4)));
        const tr_v4 c1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((tr_lds_v4*)(uintptr_t)(ad + 4 * ROWB + ((cc ^ tr_x1) << 4)));
        ct[t2] = __builtin_shufflevector(c0, c1, 0, 1, 2, 3, 4, 5, 6, 7);
      }
      __builtin_amdgcn_sched_barrier(0);
      if (next) score(t + 1);
      // ---- soft-max
      bf16x8_t pf[MH];
#pragma unroll
      for (int m = 0; m < MH; ++m) {
        float v[8];
        float mx = M_INIT_F;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          float x = raw[m][0][j >> 2][j & 3];
#pragma unroll
          for (int k = 1; k < KH; ++k) x += raw[m][k][j >> 2][j & 3];
          v[j] = k0 + 8 * g + j < hi ? x * p.scale2 : -INFINITY;
          mx = fmaxf(mx, v[j]);
        }
        mx = max_over_groups(mx);
        const float m_new = fmaxf(m_run[m], mx);
        const float alpha = fast_exp2(m_run[m] - m_new);
        m_run[m] = m_new;
        float sum = 0.f;
        u32x4 w;
#pragma unroll
        for (int j = 0; j < 8; j += 2) {
          const float e0 = fast_exp2(v[j] - m_new), e1 = fast_exp2(v[j + 1] - m_new);
          sum += e0 + e1;
          w[j >> 1] = pack2<bf16_tag>(e0, e1);
        }
        pf[m] = __builtin_bit_cast(bf16x8_t, w);
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
        for (int m = 0; m < MH; ++m)
          o[m][t2] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, ct[t2]), pf[m], o[m][t2], 0, 0, 0);
    }
    lds_barrier();   // ring and table are free for the next segment
  }

  // The accumulators (lane: head l16 of block m, latent columns 16 NT wave + 16 t + 4 g .. + 3) go through the ring, so
  // that whole lines leave the chip: straight from the registers a store touches 64 bytes of 16 rows.
  constexpr int OS = KP + 4;   // row stride (floats)
  static_assert(16 * MH * OS * 4 <= NBUF * TILE, "the output tile fits the ring");
  float* ot = reinterpret_cast<float*>(ring);
#pragma unroll
  for (int m = 0; m < MH; ++m) {
    if (columns) {
#pragma unroll
      for (int t = 0; t < NT; ++t) *reinterpret_cast<f32x4*>(ot + (16 * m + l16) * OS + wave * (16 * NT) + 16 * t + 4 * g) = o[m][t];
    }
    float l = l_run[m];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (wave == 0 && g == 0) {
      sc[0][16 * m + l16] = m_run[m];
      sc[1][16 * m + l16] = l;
    }
  }
  __syncthreads();
  const int n_heads = min(16 * MH, a.heads - h0);
  for (int i = tid; i < n_heads * (KP / 4); i += 512) {
    const int hr = i / (KP / 4), c = i % (KP / 4) * 4;
    const int64_t rh = row * a.heads + h0 + hr;
    f32x4 v = *reinterpret_cast<const f32x4*>(ot + hr * OS + c);
    if (p.n_splits == 1) {
      v *= 1.0f / sc[1][hr];  // (every row sees itself: the sum is positive)
      *reinterpret_cast<u32x2*>(reinterpret_cast<bf16*>(a.out) + rh * KP + c) =
          u32x2{pack2<bf16_tag>(v.x, v.y), pack2<bf16_tag>(v.z, v.w)};
    } else {
      *reinterpret_cast<f32x4*>(p.o_part + (rh * p.n_splits + split) * KP + c) = v;
    }
  }
  if (p.n_splits > 1 && tid < n_heads) {
    const int64_t pi = (row * a.heads + h0 + tid) * p.n_splits + split;
    p.ml_part[2 * pi] = sc[0][tid];
    p.ml_part[2 * pi + 1] = sc[1][tid];
  }
}

// Merges the splits.  A workgroup takes 256 / G groups of four columns, G threads share a group's splits.
template <int G>
__global__ void __launch_bounds__(256) latent_attn_combine_kernel(const LatentAttnK p) {
  constexpr int Q = 256 / G;
  __shared__ f32x4 part[G > 1 ? G : 1][Q];
  const int n = p.n_splits, c4 = p.a.c_pad / 4, tid = threadIdx.x;
  const int64_t quad = (int64_t)blockIdx.x * Q + tid % Q;
  if (G == 1 && quad >= p.a.rows * p.a.heads * c4) return;   // (G > 1: whole workgroups, c4 % Q == 0)
  const int64_t rh = quad / c4;
  const int c = (int)(quad % c4) * 4, sg = tid / Q;
  const float* ml = p.ml_part + 2 * rh * n;
  const float* src = p.o_part + rh * n * p.a.c_pad + c;
  float m, inv;
  if constexpr (G == 1) {
    m = M_INIT_F;
    for (int s = 0; s < n; ++s) m = fmaxf(m, ml[2 * s]);
    float l = 0.f;
    for (int s = 0; s < n; ++s) l += ml[2 * s + 1] * fast_exp2(ml[2 * s] - m);
    inv = 1.0f / l;
  } else {
    // every wave the same statistics: two splits per lane
    const int lane = tid & 63;
    const float m0 = lane < n ? ml[2 * lane] : M_INIT_F, m1 = lane + 64 < n ? ml[2 * lane + 128] : M_INIT_F;
    const float l0 = lane < n ? ml[2 * lane + 1] : 0.f, l1 = lane + 64 < n ? ml[2 * lane + 129] : 0.f;
    m = wave_max(fmaxf(m0, m1));
    inv = 1.0f / wave_sum(l0 * fast_exp2(m0 - m) + l1 * fast_exp2(m1 - m));
  }
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int s = sg; s < n; s += G) o += *reinterpret_cast<const f32x4*>(src + (int64_t)s * p.a.c_pad) * fast_exp2(ml[2 * s] - m);
  if constexpr (G > 1) {
    part[sg][tid % Q] = o;
    __syncthreads();
    if (sg) return;
#pragma unroll
    for (int s = 1; s < G; ++s) o += part[s][tid % Q];
  }
  o *= inv;
  *reinterpret_cast<u32x2*>(reinterpret_cast<bf16*>(p.a.out) + rh * p.a.c_pad + c) =
      u32x2{pack2<bf16_tag>(o.x, o.y), pack2<bf16_tag>(o.z, o.w)};
}

static void la_combine(const LatentAttnK& p, hipStream_t st) {
  const int64_t quads = p.a.rows * p.a.heads * (p.a.c_pad / 4);
  if (p.n_splits <= 8) latent_attn_combine_kernel<1><<<dim3((unsigned)((quads + 255) / 256)), dim3(256), 0, st>>>(p);
  else latent_attn_combine_kernel<16><<<dim3((unsigned)(quads / 16)), dim3(256), 0, st>>>(p);
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

// head blocks of 16 per workgroup (the scores of four do not fit beside the tiles of the widest latent)
static int la_mh(int heads, int c_pad) { return heads > 32 && c_pad < 512 ? 4 : heads > 16 ? 2 : 1; }
static bool la_mfma(int c_pad, int r_pad, int dtype) {
  return dtype == SLM_BF16 && (c_pad == 64 || c_pad == 128 || c_pad == 256 || c_pad == 512) && (r_pad == 32 || r_pad == 64);
}
static int la_splits(const slm_latent_attn_args& a) {
  if (!la_mfma(a.c_pad, a.r_pad, a.dtype) || a.generic) return 1;
  if (a.n_splits > 0) return a.n_splits < LA_MAX_SPLITS ? a.n_splits : LA_MAX_SPLITS;
  const int mh = la_mh(a.heads, a.c_pad);
  const int64_t wgs = a.rows * ((a.heads + 16 * mh - 1) / (16 * mh));
  int64_t len = a.max_kv_len > 0 ? a.max_kv_len : 1;
  if (a.window > 0 && a.window < len) len = a.window;
  const int64_t tiles = (len + LA_KT - 1) / LA_KT;
  // one round of workgroups: a ring of a wide latent fills a CU's LDS, narrow ones sit on a CU together
  const int per_cu = a.c_pad > 64 ? 1 : 2;
  int64_t n = 256 * per_cu / (wgs > 0 ? wgs : 1);
  if (n > tiles) n = tiles;
  if (n > LA_MAX_SPLITS) n = LA_MAX_SPLITS;
  return n < 1 ? 1 : (int)n;
}

template <int KP, int RP, int MH>
static void la_launch(const LatentAttnK& p, hipStream_t st) {
  const int hblocks = (p.a.heads + 16 * MH - 1) / (16 * MH);
  const int64_t groups = (p.a.rows * p.n_splits + 7) / 8;
  latent_attn_kernel<KP, RP, MH><<<dim3((unsigned)(groups * 8 * hblocks)), dim3(512), 0, st>>>(p);
}
template <int KP, int RP>
static void la_heads(const LatentAttnK& p, hipStream_t st) {
  const int mh = la_mh(p.a.heads, KP);
  if (mh == 1) la_launch<KP, RP, 1>(p, st);
  else if (mh == 2) la_launch<KP, RP, 2>(p, st);
  if constexpr (KP < 512) {
    if (mh == 4) la_launch<KP, RP, 4>(p, st);
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
    if (p.n_splits > 1) la_combine(p, st);
  } else {
    const dim3 grid((unsigned)(a->rows * a->heads));
    const size_t lds = (size_t)(a->c_pad + a->r_pad) * 4;
    if (a->dtype == SLM_BF16) latent_attn_any_kernel<bf16><<<grid, dim3(256), lds, st>>>(p);
    else latent_attn_any_kernel<float><<<grid, dim3(256), lds, st>>>(p);
  }
  return hip_check_launch();
}
