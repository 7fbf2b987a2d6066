// recurrent.hip -- layers with a matrix state S [dim, vdim] per sequence and head: the gated delta rule with a decay
// per key channel, and decayed linear attention.  Everything here is fp32 besides the projections it reads.
//
//   step     one row per sequence: convolution, activations, unit vectors, gates, the update and (delta) the output norm
//            in one launch.  One workgroup per (row, head); the state is read and written once.  Bound: HBM (state).
//   prepare  portions, cut into chunks of 16 tokens, every chunk at once: inputs activated and normed, decays summed, and
//            what a chunk's tokens do to each other solved (a 16 x 16 triangular system).  Bound: VALU, HBM.
//   scan     portions: chunk after chunk.  The columns of S are independent, so a workgroup owns 16 of them and keeps them
//            in registers from the portion's first token to its last; the products are 32-bit MFMAs.  Bound: fp32 MFMA.
//   gated_norm  the norm and gate behind a scan.
#include "latent/latent_common.h"
#include "slm_mixers.h"

namespace slm {

constexpr bool DELTA_MODE(int m) { return m == SLM_REC_DELTA; }

__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + __expf(-z)); }
// log(1 + x) = log(u) x / (u - 1) with u the rounded 1 + x: what the sum loses of x comes back (Kahan)
__device__ __forceinline__ float softplus_f32(float z) {
  const float x = __expf(-fabsf(z)), u = 1.0f + x;
  const float l = u == 1.0f ? x : __logf(u) * (x / (u - 1.0f));
  return fmaxf(z, 0.f) + l;
}
__device__ __forceinline__ float sigmoid_full(float z) { return 1.0f / (1.0f + expf(-z)); }

// the convolved, activated input of channel c (index into q | k | v) of `row` at position p; rows of the step before
// `row0` come from the ring
template <typename E>
__device__ __forceinline__ float conv_input(const slm_recurrent_args& a, const E* ring, int64_t row, int64_t row0, int p, int c) {
  const int64_t ch = 2 * (int64_t)a.qk_heads * a.dim + (int64_t)a.heads * a.vdim;
  const int qk = a.qk_heads * a.dim;
  const int64_t col = c < qk ? a.off_q + c : c < 2 * qk ? a.off_k + (c - qk) : a.off_v + (c - 2 * qk);
  const E* src = reinterpret_cast<const E*>(a.proj) + col;
  float acc = 0.f;
  for (int j = min(a.taps - 1, p); j >= 0; --j) {
    const float x = row - j >= row0 ? to_f32(src[(row - j) * a.ld_proj]) : to_f32(ring[(int64_t)((p - j) % a.taps) * ch + c]);
    acc = __builtin_fmaf(a.conv_w[(int64_t)(a.taps - 1 - j) * ch + c], x, acc);
  }
  return silu_f32(acc);
}
// (raw projection of channel c, what the ring keeps)
template <typename E>
__device__ __forceinline__ E raw_input(const slm_recurrent_args& a, int64_t row, int c) {
  const int qk = a.qk_heads * a.dim;
  const int64_t col = c < qk ? a.off_q + c : c < 2 * qk ? a.off_k + (c - qk) : a.off_v + (c - 2 * qk);
  return reinterpret_cast<const E*>(a.proj)[row * a.ld_proj + col];
}
// the same for the 16 tokens from `row` on (n of them there are), convolutions of at most 4 taps: every input is read once
template <typename E, typename F>
__device__ __forceinline__ void conv_run4(const slm_recurrent_args& a, const E* ring, int64_t row, int64_t row0, int p, int n, int c, F put) {
  const int64_t ch = 2 * (int64_t)a.qk_heads * a.dim + (int64_t)a.heads * a.vdim;
  const int qk = a.qk_heads * a.dim;
  const int64_t col = c < qk ? a.off_q + c : c < 2 * qk ? a.off_k + (c - qk) : a.off_v + (c - 2 * qk);
  const E* src = reinterpret_cast<const E*>(a.proj) + row * a.ld_proj + col;
  float w[4], x[19];   // w[j]: of the input j tokens back; x[3 + t]: the input of token t
#pragma unroll
  for (int j = 0; j < 4; ++j) w[j] = j < a.taps ? a.conv_w[(int64_t)(a.taps - 1 - j) * ch + c] : 0.f;
#pragma unroll
  for (int j = 1; j < 4; ++j) {
    x[3 - j] = 0.f;
    if (j < a.taps && p >= j)
      x[3 - j] = row - j >= row0 ? to_f32(src[-j * a.ld_proj]) : to_f32(ring[(int64_t)((p - j) % a.taps) * ch + c]);
  }
#pragma unroll
  for (int t = 0; t < 16; ++t) x[3 + t] = to_f32(src[min(t, n - 1) * a.ld_proj]);
#pragma unroll
  for (int t = 0; t < 16; ++t) {
    float acc = w[3] * x[t];
#pragma unroll
    for (int j = 2; j >= 0; --j) acc = __builtin_fmaf(w[j], x[3 + t - j], acc);
    put(t, t < n ? silu_f32(acc) : 0.f);
  }
}
template <typename E>
__device__ __forceinline__ float decay_exponent(const slm_recurrent_args& a, int64_t row, int head, int c) {
  const float x = to_f32(reinterpret_cast<const E*>(a.low)[row * a.ld_low + (int64_t)head * a.dim + c]);
  return a.neg_a[head] * softplus_f32(x + a.dt_bias[head * a.dim + c]);
}

// ---------------------------------------------------------------------------------------
// step: threads = 256 per 64 columns; thread = (4 columns, row group of 16), NR rows of its group
// ---------------------------------------------------------------------------------------
template <typename E, int MODE, int NR>
__global__ void __launch_bounds__(1024) recurrent_step_kernel(const slm_recurrent_args a) {
  constexpr int DK = 16 * NR;
  __shared__ float sq[DK], sk[DK], sg[DK], sv[256], red[16][64], wred[2][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int nthreads = blockDim.x, n_waves = nthreads >> 6;
  const int head = blockIdx.x % a.heads;
  const int64_t row = blockIdx.x / a.heads;
  const int p = a.positions[row];
  const int slot = a.state_slots[row];
  const int qh = head / (a.heads / a.qk_heads);
  const int colq = (lane & 15) + 16 * (wave >> 2);
  const int rg = (wave & 3) * 4 + (lane >> 4);
  const bool mine = 4 * colq < a.v_pad;
  float* S = a.state + ((int64_t)slot * a.heads + head) * DK * a.v_pad + 4 * colq;

  f32x4 s[NR];
#pragma unroll
  for (int r = 0; r < NR; ++r)
    s[r] = mine && p > 0 ? *reinterpret_cast<const f32x4*>(S + (int64_t)(rg + 16 * r) * a.v_pad) : f32x4{0.f, 0.f, 0.f, 0.f};

  float beta = 0.f;
  if constexpr (DELTA_MODE(MODE)) {
    const int64_t ch = 2 * (int64_t)a.qk_heads * a.dim + (int64_t)a.heads * a.vdim;
    const int qk = a.qk_heads * a.dim;
    E* ring = reinterpret_cast<E*>(a.conv_ring) + (int64_t)slot * a.taps * ch;
    E* keep = ring + (int64_t)(p % a.taps) * ch;   // (no head reads this entry: the ring holds one more than the history)
    const bool first_of_group = head % (a.heads / a.qk_heads) == 0;
    float nq = 0.f, nk = 0.f;
    for (int i = tid; i < DK; i += nthreads) {
      float q = 0.f, k = 0.f, g = 0.f;
      if (i < a.dim) {
        const int c = qh * a.dim + i;
        q = conv_input<E>(a, ring, row, row, p, c);
        k = conv_input<E>(a, ring, row, row, p, qk + c);
        g = expf(decay_exponent<E>(a, row, head, i));
        if (first_of_group) {
          keep[c] = raw_input<E>(a, row, c);
          keep[qk + c] = raw_input<E>(a, row, qk + c);
        }
      }
      nq = __builtin_fmaf(q, q, nq);
      nk = __builtin_fmaf(k, k, nk);
      sq[i] = q, sk[i] = k, sg[i] = g;
    }
    for (int i = nthreads - 1 - tid; i < a.v_pad; i += nthreads) {
      float v = 0.f;
      if (i < a.vdim) {
        const int c = 2 * qk + head * a.vdim + i;
        v = conv_input<E>(a, ring, row, row, p, c);
        keep[c] = raw_input<E>(a, row, c);
      }
      sv[i] = v;
    }
    nq = wave_sum(nq), nk = wave_sum(nk);
    if (lane == 0) wred[0][wave] = nq, wred[1][wave] = nk;
    __syncthreads();
    nq = nk = 0.f;
    for (int w = 0; w < n_waves; ++w) nq += wred[0][w], nk += wred[1][w];
    const float fq = a.q_scale / sqrtf(nq + a.unit_eps), fk = 1.0f / sqrtf(nk + a.unit_eps);
    beta = sigmoid_full(to_f32(reinterpret_cast<const E*>(a.proj)[row * a.ld_proj + a.off_b + head]));
    float kv[4] = {0.f, 0.f, 0.f, 0.f}, ks[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const float g = sg[rg + 16 * r];
      ks[r] = sk[rg + 16 * r] * fk;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[r][j] *= g;
        kv[j] = __builtin_fmaf(ks[r], s[r][j], kv[j]);
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      kv[j] += __shfl_xor(kv[j], 16, 64);
      kv[j] += __shfl_xor(kv[j], 32, 64);
    }
    if (lane < 16) *reinterpret_cast<f32x4*>(&red[wave][4 * lane]) = f32x4{kv[0], kv[1], kv[2], kv[3]};
    __syncthreads();
    float o[4] = {0.f, 0.f, 0.f, 0.f}, u[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float t = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) t += red[(wave & ~3) + w][4 * (lane & 15) + j];
      u[j] = mine ? beta * (sv[4 * colq + j] - t) : 0.f;
    }
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const float q = sq[rg + 16 * r] * fq;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[r][j] = __builtin_fmaf(ks[r], u[j], s[r][j]);
        o[j] = __builtin_fmaf(q, s[r][j], o[j]);
      }
    }
    if (mine)
#pragma unroll
      for (int r = 0; r < NR; ++r) *reinterpret_cast<f32x4*>(S + (int64_t)(rg + 16 * r) * a.v_pad) = s[r];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      o[j] += __shfl_xor(o[j], 16, 64);
      o[j] += __shfl_xor(o[j], 32, 64);
    }
    __syncthreads();
    if (lane < 16) *reinterpret_cast<f32x4*>(&red[wave][4 * lane]) = f32x4{o[0], o[1], o[2], o[3]};
    __syncthreads();
    // read-out: norm over vdim, weight, gate (threads 0 .. v_pad - 1 hold a column each)
    float x = 0.f;
    if (tid < a.v_pad) {
      const int w0 = 4 * (tid >> 6);
#pragma unroll
      for (int w = 0; w < 4; ++w) x += red[w0 + w][tid & 63];
    }
    const float ss = wave_sum(x * x);
    if (lane == 0) wred[0][wave] = ss;
    __syncthreads();
    float total = 0.f;
    for (int w = 0; w < n_waves; ++w) total += wred[0][w];
    const float rs = 1.0f / sqrtf(total / (float)a.vdim + a.eps);
    E* out = reinterpret_cast<E*>(a.out) + row * a.ld_out;
    if (tid < a.vdim) {
      const float gate = to_f32(reinterpret_cast<const E*>(a.low)[row * a.ld_low + a.off_gate + (int64_t)head * a.vdim + tid]);
      out[head * a.vdim + tid] = (E)(x * rs * a.norm_weight[tid] * sigmoid_f32(gate));
    }
    if (head == a.heads - 1)
      for (int64_t i = (int64_t)a.heads * a.vdim + tid; i < a.ld_out; i += nthreads) out[i] = (E)0.f;
  } else {
    const E* pr = reinterpret_cast<const E*>(a.proj) + row * a.ld_proj;
    for (int i = tid; i < DK; i += nthreads) {
      sq[i] = i < a.dim ? silu_f32(to_f32(pr[a.off_q + qh * a.dim + i])) : 0.f;
      sk[i] = i < a.dim ? silu_f32(to_f32(pr[a.off_k + qh * a.dim + i])) : 0.f;
    }
    for (int i = nthreads - 1 - tid; i < a.v_pad; i += nthreads) sv[i] = i < a.vdim ? silu_f32(to_f32(pr[a.off_v + head * a.vdim + i])) : 0.f;
    __syncthreads();
    const float d = a.decay[head];
    float o[4] = {0.f, 0.f, 0.f, 0.f}, v[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = mine ? sv[4 * colq + j] : 0.f;
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      const float k = sk[rg + 16 * r], q = sq[rg + 16 * r];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[r][j] = __builtin_fmaf(k, v[j], s[r][j] * d);
        o[j] = __builtin_fmaf(q, s[r][j], o[j]);
      }
      if (mine) *reinterpret_cast<f32x4*>(S + (int64_t)(rg + 16 * r) * a.v_pad) = s[r];
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      o[j] += __shfl_xor(o[j], 16, 64);
      o[j] += __shfl_xor(o[j], 32, 64);
    }
    if (lane < 16) *reinterpret_cast<f32x4*>(&red[wave][4 * lane]) = f32x4{o[0], o[1], o[2], o[3]};
    __syncthreads();
    if (tid < a.v_pad) {
      const int w0 = 4 * (tid >> 6);
      float x = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) x += red[w0 + w][tid & 63];
      a.o[(row * a.heads + head) * a.v_pad + tid] = x;
    }
  }
}

// ---------------------------------------------------------------------------------------
// portions: chunks of 16 tokens
// ---------------------------------------------------------------------------------------
// With L_t the sum of a chunk's log decays up to token t, S0 the state in front of it, x.d = product per key channel:
//   (I + diag(beta) A) U = diag(beta) (V - Kd S0)     A_ts = sum_d k_t k_s exp(L_t - L_s), s < t;  Kd_t = k_t exp(L_t)
//   O  = Qd S0 + B U                                  B_ts = sum_d q_t k_s exp(L_t - L_s), s <= t; Qd_t = q_t exp(L_t)
//   S1 = diag(exp(L_end)) S0 + Kr^T U                 Kr_t = k_t exp(L_end - L_t)
// Every exponent is <= 0: nothing overflows however fast a channel forgets.  Without the delta rule U = V.
// A chunk's record for one head, in floats:
//   Kd | Qd (16 x DK each) | Kr^T (DK x 16) | exp(L_end) (DK) | V^T (v_pad x 16) | T = (I + diag(beta) A)^-1 diag(beta) | B (16 x 16)
// Matrices are tiles of 16 x 16 in the order the scan's lanes take them, four floats a lane: entry (m, k) at
// tile_at(m, k), so that a wave reads a tile as 1 KiB in a row.  Kd, Qd: m token, k channel; Kr^T, V^T: m channel / column,
// k token; T, B: m row, k column.
__device__ __forceinline__ int tile_at(int m, int k) { return (((k >> 2) & 3) * 16 + (m & 15)) * 4 + (k & 3); }
template <int DK>
struct ChunkRecord {
  static constexpr int KD = 0, QD = 16 * DK, KR = 32 * DK, GE = 48 * DK, V = 49 * DK;
  int v_pad;
  __device__ __forceinline__ int t() const { return V + 16 * v_pad; }
  __device__ __forceinline__ int b() const { return t() + 256; }
  __device__ __forceinline__ int64_t size() const { return b() + 256; }
};

// one workgroup per (chunk, head); every chunk of the step at once
template <typename E, int MODE, int DK>
__global__ void __launch_bounds__(256) recurrent_prepare_kernel(const slm_recurrent_args a) {
  constexpr bool DELTA = DELTA_MODE(MODE);
  constexpr int LD = DK + 4;                     // (the 16 rows a quarter-wave reads by 16 bytes are in different banks)
  __shared__ __attribute__((aligned(16))) float sq[16 * LD], sk[16 * LD], sL[16 * LD];
  __shared__ float sa[16][17], sbeta[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int head = blockIdx.x % a.heads;
  const int64_t chunk = blockIdx.x / a.heads;
  const int32_t* cd = a.chunks + 3 * chunk;
  const int seq = cd[0], n = cd[2];
  const int64_t row = cd[1], row0 = a.q_cu[seq];
  const int p = a.positions[row];
  const int qh = head / (a.heads / a.qk_heads), qk = a.qk_heads * a.dim;
  const ChunkRecord<DK> at{a.v_pad};
  float* rec = a.pre + (chunk * a.heads + head) * at.size();
  const E* ring = nullptr;
  if constexpr (DELTA)
    ring = reinterpret_cast<const E*>(a.conv_ring) + (int64_t)a.state_slots[seq] * a.taps * (2 * (int64_t)qk + (int64_t)a.heads * a.vdim);
  const E* in = reinterpret_cast<const E*>(a.proj) + row * a.ld_proj;
  const float step_l = DELTA ? 0.f : fmaxf(log2f(a.decay[head]), -126.f);

  if (DELTA && a.taps <= 4) {
    for (int i = tid; i < 2 * DK + a.v_pad; i += 256) {
      if (i < 2 * DK) {
        const int c = i < DK ? i : i - DK;
        float* dst = (i < DK ? sq : sk) + c;
        auto put = [&](int t, float x) { dst[t * LD] = x; };
        if (c < a.dim) {
          conv_run4<E>(a, ring, row, row0, p, n, (i < DK ? 0 : qk) + qh * a.dim + c, put);
        } else {
#pragma unroll
          for (int t = 0; t < 16; ++t) put(t, 0.f);
        }
      } else {
        const int c = i - 2 * DK;
        float* dst = rec + ChunkRecord<DK>::V + (c >> 4) * 256 + (c & 15) * 4;
        f32x4 four;
        auto put = [&](int t, float x) {
          four[t & 3] = x;
          if ((t & 3) == 3) *reinterpret_cast<f32x4*>(dst + (t >> 2) * 64) = four;
        };
        if (c < a.vdim) {
          conv_run4<E>(a, ring, row, row0, p, n, 2 * qk + head * a.vdim + c, put);
        } else {
#pragma unroll
          for (int t = 0; t < 16; ++t) put(t, 0.f);
        }
      }
    }
  } else {
    for (int i = tid; i < 16 * DK; i += 256) {
      const int t = i / DK, c = i % DK;
      float q = 0.f, k = 0.f;
      if (t < n && c < a.dim) {
        if constexpr (DELTA) {
          q = conv_input<E>(a, ring, row + t, row0, p + t, qh * a.dim + c);
          k = conv_input<E>(a, ring, row + t, row0, p + t, qk + qh * a.dim + c);
        } else {
          q = silu_f32(to_f32(in[t * a.ld_proj + a.off_q + qh * a.dim + c]));
          k = silu_f32(to_f32(in[t * a.ld_proj + a.off_k + qh * a.dim + c]));
        }
      }
      sq[t * LD + c] = q, sk[t * LD + c] = k;
    }
    for (int i = tid; i < 16 * a.v_pad; i += 256) {   // (in the record's order)
      const int t = ((i >> 6) & 3) * 4 + (i & 3), c = (i >> 8) * 16 + ((i >> 2) & 15);
      float v = 0.f;
      if (t < n && c < a.vdim) {
        if constexpr (DELTA) v = conv_input<E>(a, ring, row + t, row0, p + t, 2 * qk + head * a.vdim + c);
        else v = silu_f32(to_f32(in[t * a.ld_proj + a.off_v + head * a.vdim + c]));
      }
      rec[ChunkRecord<DK>::V + i] = v;
    }
  }
  for (int i = tid; i < 16 * DK; i += 256) {
    const int t = i / DK, c = i % DK;
    float l = 0.f;
    if (t < n && c < a.dim) {
      if constexpr (DELTA) l = LOG2E_F * decay_exponent<E>(a, row + t, head, c);
      else l = step_l;
    }
    sL[t * LD + c] = l;
  }
  if (DELTA && tid < 16) sbeta[tid] = tid < n ? sigmoid_full(to_f32(in[tid * a.ld_proj + a.off_b + head])) : 0.f;
  __syncthreads();
  if constexpr (DELTA) {   // unit vectors: four tokens per wave
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int t = 4 * wave + j;
      float nq = 0.f, nk = 0.f;
      for (int c = lane; c < DK; c += 64) {
        nq = __builtin_fmaf(sq[t * LD + c], sq[t * LD + c], nq);
        nk = __builtin_fmaf(sk[t * LD + c], sk[t * LD + c], nk);
      }
      const float fq = a.q_scale / sqrtf(wave_sum(nq) + a.unit_eps), fk = 1.0f / sqrtf(wave_sum(nk) + a.unit_eps);
      for (int c = lane; c < DK; c += 64) sq[t * LD + c] *= fq, sk[t * LD + c] *= fk;
    }
  }
  if (tid < DK) {
    float l = 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      l += sL[t * LD + tid];
      sL[t * LD + tid] = l;
    }
  }
  __syncthreads();
  {
    const int t = tid >> 4, s = tid & 15;
    float x = 0.f, y = 0.f;
    if (s <= t) {
      if constexpr (DELTA) {
#pragma unroll 2
        for (int c = 0; c < DK; c += 4) {
          const f32x4 ks = *reinterpret_cast<const f32x4*>(sk + s * LD + c), ls = *reinterpret_cast<const f32x4*>(sL + s * LD + c);
          const f32x4 kt = *reinterpret_cast<const f32x4*>(sk + t * LD + c), lt = *reinterpret_cast<const f32x4*>(sL + t * LD + c);
          const f32x4 qt = *reinterpret_cast<const f32x4*>(sq + t * LD + c);
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float e = ks[j] * fast_exp2(lt[j] - ls[j]);
            x = __builtin_fmaf(kt[j], e, x);
            y = __builtin_fmaf(qt[j], e, y);
          }
        }
      } else {
#pragma unroll 2
        for (int c = 0; c < DK; c += 4) {
          const f32x4 ks = *reinterpret_cast<const f32x4*>(sk + s * LD + c), qt = *reinterpret_cast<const f32x4*>(sq + t * LD + c);
#pragma unroll
          for (int j = 0; j < 4; ++j) y = __builtin_fmaf(qt[j], ks[j], y);
        }
        y *= fast_exp2(sL[t * LD] - sL[s * LD]);
      }
    }
    rec[at.b() + tile_at(t, s)] = y;
    sa[t][s] = x;
  }
  for (int i = tid; i < 4 * DK; i += 256) {   // four floats each, in the record's order
    const int tile = i >> 6, m = i & 15, k = ((i >> 4) & 3) * 4;
    {
      const int at_t = m * LD + 16 * tile + k;
      const f32x4 l = *reinterpret_cast<const f32x4*>(sL + at_t), q = *reinterpret_cast<const f32x4*>(sq + at_t);
      const f32x4 e = {fast_exp2(l.x), fast_exp2(l.y), fast_exp2(l.z), fast_exp2(l.w)};
      if constexpr (DELTA) *reinterpret_cast<f32x4*>(rec + ChunkRecord<DK>::KD + 4 * i) = *reinterpret_cast<const f32x4*>(sk + at_t) * e;
      *reinterpret_cast<f32x4*>(rec + ChunkRecord<DK>::QD + 4 * i) = q * e;
    }
    const int d = 16 * tile + m;
    f32x4 kr;
#pragma unroll
    for (int j = 0; j < 4; ++j) kr[j] = sk[(k + j) * LD + d] * fast_exp2(sL[15 * LD + d] - sL[(k + j) * LD + d]);
    *reinterpret_cast<f32x4*>(rec + ChunkRecord<DK>::KR + 4 * i) = kr;
  }
  if (tid < DK) rec[ChunkRecord<DK>::GE + tid] = fast_exp2(sL[15 * LD + tid]);
  if constexpr (DELTA) {
    __syncthreads();
    if (tid < 16) {   // column tid of T by forward substitution
      float x[16];
#pragma unroll
      for (int t = 0; t < 16; ++t) {
        float v = t == tid ? 1.0f : 0.f;
#pragma unroll
        for (int s = 0; s < t; ++s) v = __builtin_fmaf(-sa[t][s], x[s], v);
        x[t] = sbeta[t] * v;
        rec[at.t() + tile_at(t, tid)] = x[t];
      }
    }
  }
}

// One workgroup per (sequence, head, 16 NCT columns of S), chunk after chunk.  Its waves share the key channels: a wave
// keeps TPW tiles [16 x 16] of every column tile of S in registers in the accumulator layout of the 32-bit MFMA (row 4 g + r,
// column l16), which is the layout its right operand takes when the contraction index of product r is 4 g + r.  Partial
// products with S0 meet in LDS, one barrier a chunk; U is computed by every wave; read-outs are completed a chunk later.  The operands of the next chunks travel
// meanwhile.  Two column tiles read the records half as often: where enough workgroups are left.
template <int TPW, int NCT>
struct ChunkOperands {
  f32x4 kd[TPW], qd[TPW], kr[TPW], ge[TPW], t, b, v[NCT];
};

template <typename E, int MODE, int DK, int W, int NCT>
__global__ void __launch_bounds__(64 * W, 2) recurrent_scan_kernel(const slm_recurrent_args a) {
  constexpr bool DELTA = DELTA_MODE(MODE);
  constexpr int TPW = DK / 16 / W;
  constexpr int NB = TPW <= (DELTA ? 1 : 2) ? 3 : 2;   // chunks in registers: one in use, the others on their way
  __shared__ f32x4 part_u[2][NCT][W][64], part_o[2][NCT][W][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l16 = lane & 15, g = lane >> 4;
  // the column blocks of one head on one XCD (workgroups go round the XCDs): they read the same records
  const int n_ct = a.v_pad / 16, n_cb = (n_ct + NCT - 1) / NCT, n_items = (a.batch - a.n_single) * a.heads;
  const int cb = blockIdx.x / 8 % n_cb, item = blockIdx.x / (8 * n_cb) * 8 + blockIdx.x % 8;
  if (item >= n_items) return;
  const int head = item % a.heads, ps = item / a.heads, seq = a.n_single + ps;
  const int64_t row0 = a.q_cu[seq];
  const int n = a.q_cu[seq + 1] - (int)row0;
  const int p0 = a.positions[row0], slot = a.state_slots[seq];
  const int64_t chunk0 = a.seq_chunks[ps];
  const int n_chunks = (n + 15) / 16;
  const ChunkRecord<DK> at{a.v_pad};
  const float* rec0 = a.pre + (chunk0 * a.heads + head) * at.size();
  const int64_t rec_step = a.heads * at.size();
  float* S = a.state + (((int64_t)slot * a.heads + head) * DK + 16 * TPW * wave + 4 * g) * a.v_pad + l16;
  int ct[NCT];   // (an odd last tile is computed twice and stored once)
#pragma unroll
  for (int j = 0; j < NCT; ++j) ct[j] = min(cb * NCT + j, n_ct - 1);

  f32x4 s[NCT][TPW];
#pragma unroll
  for (int j = 0; j < NCT; ++j)
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) s[j][i][r] = p0 > 0 ? S[(int64_t)(16 * i + r) * a.v_pad + 16 * ct[j]] : 0.f;

  // uniform bases and 32-bit lane offsets: an address is one register
  auto vec = [](const float* base, uint32_t off) { return *reinterpret_cast<const f32x4*>(reinterpret_cast<const char*>(base) + off); };
  const uint32_t off = (uint32_t)lane * 16, ge_off = (uint32_t)g * 16;
  auto load = [&](int c, ChunkOperands<TPW, NCT>& x) {
    const float* rec = rec0 + c * rec_step;
#pragma unroll
    for (int i = 0; i < TPW; ++i) {
      const int tile = TPW * wave + i;
      if constexpr (DELTA) x.kd[i] = vec(rec + ChunkRecord<DK>::KD + 256 * tile, off);
      x.qd[i] = vec(rec + ChunkRecord<DK>::QD + 256 * tile, off);
      x.kr[i] = vec(rec + ChunkRecord<DK>::KR + 256 * tile, off);
      x.ge[i] = vec(rec + ChunkRecord<DK>::GE + 16 * tile, ge_off);
    }
    if constexpr (DELTA) x.t = vec(rec + at.t(), off);
    x.b = vec(rec + at.b(), off);
#pragma unroll
    for (int j = 0; j < NCT; ++j) x.v[j] = vec(rec + ChunkRecord<DK>::V + 256 * ct[j], off);
  };
  auto mma4 = [](const f32x4& x, const f32x4& y, f32x4 c) {
#pragma unroll
    for (int r = 0; r < 4; ++r) c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[r], y[r], c, 0, 0, 0);
    return c;
  };
  auto finish = [&](int c) {   // the read-outs of chunk c, once every wave's part of them is there
#pragma unroll
    for (int j = 0; j < NCT; ++j)
      if ((c * NCT + j + W / 2) % W == wave && cb * NCT + j < n_ct) {
        f32x4 y = part_o[c & 1][j][0][lane];
#pragma unroll
        for (int w = 1; w < W; ++w) y += part_o[c & 1][j][w][lane];
        float* dst = a.o + ((row0 - a.n_single + 16 * c) * a.heads + head) * a.v_pad + 16 * ct[j];
        const uint32_t o_off = (uint32_t)(4 * g * a.heads * a.v_pad + l16) * 4;
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (16 * c + 4 * g + r < n)
            *reinterpret_cast<float*>(reinterpret_cast<char*>(dst + (int64_t)r * a.heads * a.v_pad) + o_off) = y[r];
      }
  };
  auto chunk = [&](int c, const ChunkOperands<TPW, NCT>& x) {
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    const int b = c & 1;
    f32x4 kr[NCT], o[NCT], u[NCT];
#pragma unroll
    for (int j = 0; j < NCT; ++j) kr[j] = o[j] = zero;
    if constexpr (DELTA) {
#pragma unroll
      for (int i = 0; i < TPW; ++i)
#pragma unroll
        for (int j = 0; j < NCT; ++j) kr[j] = mma4(x.kd[i], s[j][i], kr[j]);
#pragma unroll
      for (int j = 0; j < NCT; ++j) part_u[b][j][wave][lane] = kr[j];
    }
    // (what the next chunk does not wait for runs under the exchange)
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int j = 0; j < NCT; ++j) o[j] = mma4(x.qd[i], s[j][i], o[j]);
    lds_barrier();
#pragma unroll
    for (int j = 0; j < NCT; ++j) {
      u[j] = x.v[j];
      if constexpr (DELTA) {
#pragma unroll
        for (int w = 0; w < W; ++w) u[j] -= part_u[b][j][w][lane];
        u[j] = mma4(x.t, u[j], zero);
      }
    }
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int j = 0; j < NCT; ++j) s[j][i] = mma4(x.kr[i], u[j], s[j][i] * x.ge[i]);
#pragma unroll
    for (int j = 0; j < NCT; ++j) {   // (the waves take B U, and the stores a barrier later, in turn)
      if ((c * NCT + j) % W == wave) o[j] = mma4(x.b, u[j], o[j]);
      part_o[b][j][wave][lane] = o[j];
    }
    if (c > 0) finish(c - 1);
  };
  ChunkOperands<TPW, NCT> x[NB];
#pragma unroll
  for (int i = 0; i + 1 < NB; ++i) load(min(i, n_chunks - 1), x[i]);
  int c0 = 0;   // (whole rounds without a branch around the loads: a join would make every wait one for the youngest)
  for (; c0 + NB <= n_chunks; c0 += NB) {
#pragma unroll
    for (int i = 0; i < NB; ++i) {
      load(min(c0 + i + NB - 1, n_chunks - 1), x[(i + NB - 1) % NB]);
      chunk(c0 + i, x[i]);
    }
  }
#pragma unroll
  for (int i = 0; i + 1 < NB; ++i)
    if (c0 + i < n_chunks) chunk(c0 + i, x[i]);
  lds_barrier();
  finish(n_chunks - 1);
#pragma unroll
  for (int j = 0; j < NCT; ++j)
    if (cb * NCT + j < n_ct)
#pragma unroll
      for (int i = 0; i < TPW; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[(int64_t)(16 * i + r) * a.v_pad + 16 * ct[j]] = s[j][i][r];

  // the last inputs of the convolutions (their readers ran in the launch before)
  if (DELTA && cb == 0) {
    const int qh = head / (a.heads / a.qk_heads), qk = a.qk_heads * a.dim;
    const int64_t ch = 2 * (int64_t)qk + (int64_t)a.heads * a.vdim;
    E* ring = reinterpret_cast<E*>(a.conv_ring) + (int64_t)slot * a.taps * ch;
    const bool first_of_group = head % (a.heads / a.qk_heads) == 0;
    for (int j = max(0, n - a.taps); j < n; ++j) {
      E* dst = ring + (int64_t)((p0 + j) % a.taps) * ch;
      if (first_of_group)
        for (int i = tid; i < a.dim; i += 64 * W) {
          dst[qh * a.dim + i] = raw_input<E>(a, row0 + j, qh * a.dim + i);
          dst[qk + qh * a.dim + i] = raw_input<E>(a, row0 + j, qk + qh * a.dim + i);
        }
      for (int i = tid; i < a.vdim; i += 64 * W) dst[2 * qk + head * a.vdim + i] = raw_input<E>(a, row0 + j, 2 * qk + head * a.vdim + i);
    }
  }
}

// ---------------------------------------------------------------------------------------
// gated norm: WAVES waves per group
// ---------------------------------------------------------------------------------------
template <typename E, bool PER_HEAD>
__global__ void __launch_bounds__(256) gated_norm_kernel(const slm_gated_norm_args a) {
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid & 63;
  if constexpr (PER_HEAD) {
    const int64_t item = (int64_t)blockIdx.x * 4 + (tid >> 6);
    if (item >= a.rows * a.heads) return;
    const int64_t row = item / a.heads;
    const int h = item % a.heads;
    const float* o = a.o + item * a.v_pad;
    const E* gate = reinterpret_cast<const E*>(a.gate) + row * a.ld_gate + (int64_t)h * a.vdim;
    E* out = reinterpret_cast<E*>(a.out) + row * a.ld_out;
    float x[4], gl[4], w[4], ss = 0.f;   // (v_pad <= 256)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int c = lane + 64 * j;
      const bool in = c < a.vdim;
      x[j] = in ? o[c] : 0.f, gl[j] = in ? to_f32(gate[c]) : 0.f, w[j] = in ? a.weight[c] : 0.f;
      ss = __builtin_fmaf(x[j], x[j], ss);
    }
    const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (lane + 64 * j < a.vdim) out[h * a.vdim + lane + 64 * j] = (E)(a.scale * x[j] * rs * w[j] * sigmoid_f32(gl[j]));
    if (h == a.heads - 1)
      for (int64_t c = (int64_t)a.heads * a.vdim + lane; c < a.out_width; c += 64) out[c] = (E)0.f;
  } else {
    const int64_t row = blockIdx.x;
    const int n = a.heads * a.vdim;
    const float* o = a.o + row * a.heads * a.v_pad;
    const bool packed = a.vdim == a.v_pad;
    auto at = [&](int i) { return packed ? o[i] : o[i / a.vdim * a.v_pad + i % a.vdim]; };
    float ss = 0.f;
    for (int i = tid; i < n; i += 256) {
      const float x = at(i);
      ss = __builtin_fmaf(x, x, ss);
    }
    const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)n + a.eps);
    const E* gate = reinterpret_cast<const E*>(a.gate) + row * a.ld_gate;
    E* out = reinterpret_cast<E*>(a.out) + row * a.ld_out;
    for (int i = tid; i < n; i += 256) out[i] = (E)(a.scale * at(i) * rs * a.weight[i] * sigmoid_f32(to_f32(gate[i])));
    for (int64_t i = n + tid; i < a.out_width; i += 256) out[i] = (E)0.f;
  }
}

constexpr int64_t NCT2_MIN = 512;   // column tiles from which a workgroup takes two
static bool rec_sizes_ok(const slm_recurrent_args& a) {
  return a.heads > 0 && a.qk_heads > 0 && a.heads % a.qk_heads == 0 && a.dim > 0 && a.vdim > 0 && a.vdim <= a.v_pad &&
         a.v_pad % 16 == 0 && a.v_pad <= 256 && a.dim_pad >= a.dim && a.dim_pad == slm_recurrent_dim_pad(a.dim) &&
         (a.mode == SLM_REC_DELTA || a.mode == SLM_REC_LIGHTNING) && (a.dtype == SLM_BF16 || a.dtype == SLM_F32) &&
         a.batch >= 1 && a.n_single >= 0 && a.n_single <= a.batch && a.rows >= a.n_single && a.rows <= 0x7fffffff;
}
static bool rec_ptrs_ok(const slm_recurrent_args& a) {
  if (!a.proj || !a.state || !a.positions || !a.q_cu || !a.state_slots || !aligned16(a.state)) return false;
  if (a.mode == SLM_REC_LIGHTNING) return a.decay != nullptr;
  return a.low && a.conv_w && a.conv_ring && a.neg_a && a.dt_bias && a.taps >= 1;
}

template <typename E, int MODE>
static int rec_step(const slm_recurrent_args& a, hipStream_t st) {
  const dim3 grid((unsigned)((int64_t)a.n_single * a.heads)), block(256 * ((a.v_pad + 63) / 64));
  hip_clear_error();
  switch (a.dim_pad / 16) {
    case 2: recurrent_step_kernel<E, MODE, 2><<<grid, block, 0, st>>>(a); break;
    case 4: recurrent_step_kernel<E, MODE, 4><<<grid, block, 0, st>>>(a); break;
    case 8: recurrent_step_kernel<E, MODE, 8><<<grid, block, 0, st>>>(a); break;
    case 12: recurrent_step_kernel<E, MODE, 12><<<grid, block, 0, st>>>(a); break;
    default: recurrent_step_kernel<E, MODE, 16><<<grid, block, 0, st>>>(a);
  }
  return hip_check_launch();
}
template <typename E, int MODE, int DK, int NCT>
static void rec_scan_nct(const slm_recurrent_args& a, hipStream_t st) {
  constexpr int W = DK / 16 < 4 ? DK / 16 : 4;
  const int64_t items = (int64_t)(a.batch - a.n_single) * a.heads, n_cb = (a.v_pad / 16 + NCT - 1) / NCT;
  recurrent_scan_kernel<E, MODE, DK, W, NCT><<<dim3((unsigned)((items + 7) / 8 * 8 * n_cb)), dim3(64 * W), 0, st>>>(a);
}
template <typename E, int MODE, int DK>
static void rec_scan_dk(const slm_recurrent_args& a, hipStream_t st) {
  if (DK <= 128 && (int64_t)(a.batch - a.n_single) * a.heads * (a.v_pad / 16) >= NCT2_MIN) rec_scan_nct<E, MODE, DK, (DK <= 128 ? 2 : 1)>(a, st);
  else rec_scan_nct<E, MODE, DK, 1>(a, st);
}
template <typename E, int MODE>
static int rec_scan(const slm_recurrent_args& a, hipStream_t st) {
  hip_clear_error();
  switch (a.dim_pad) {
    case 32: rec_scan_dk<E, MODE, 32>(a, st); break;
    case 64: rec_scan_dk<E, MODE, 64>(a, st); break;
    case 128: rec_scan_dk<E, MODE, 128>(a, st); break;
    case 192: rec_scan_dk<E, MODE, 192>(a, st); break;
    default: rec_scan_dk<E, MODE, 256>(a, st);
  }
  return hip_check_launch();
}
template <typename E, int MODE>
static int rec_prepare(const slm_recurrent_args& a, hipStream_t st) {
  const dim3 grid((unsigned)((int64_t)a.n_chunks * a.heads)), block(256);
  hip_clear_error();
  switch (a.dim_pad) {
    case 32: recurrent_prepare_kernel<E, MODE, 32><<<grid, block, 0, st>>>(a); break;
    case 64: recurrent_prepare_kernel<E, MODE, 64><<<grid, block, 0, st>>>(a); break;
    case 128: recurrent_prepare_kernel<E, MODE, 128><<<grid, block, 0, st>>>(a); break;
    case 192: recurrent_prepare_kernel<E, MODE, 192><<<grid, block, 0, st>>>(a); break;
    default: recurrent_prepare_kernel<E, MODE, 256><<<grid, block, 0, st>>>(a);
  }
  return hip_check_launch();
}

}  // namespace slm

using namespace slm;

extern "C" SLM_API int32_t slm_recurrent_dim_pad(int32_t dim) {
  const int32_t w[] = {32, 64, 128, 192, 256};
  for (int32_t x : w)
    if (dim > 0 && dim <= x) return x;
  return 0;
}
#define SLM_REC_DISPATCH(fn)                                                                                               \
  hipStream_t st = (hipStream_t)stream;                                                                                    \
  if (a->mode == SLM_REC_DELTA) return a->dtype == SLM_BF16 ? fn<bf16, SLM_REC_DELTA>(*a, st) : fn<float, SLM_REC_DELTA>(*a, st); \
  return a->dtype == SLM_BF16 ? fn<bf16, SLM_REC_LIGHTNING>(*a, st) : fn<float, SLM_REC_LIGHTNING>(*a, st);

extern "C" SLM_API int slm_recurrent_step(const slm_recurrent_args* a, void* stream) {
  if (!a || !rec_sizes_ok(*a) || !rec_ptrs_ok(*a)) return SLM_ERR_INVALID_ARG;
  if (a->mode == SLM_REC_DELTA ? (!a->out || !a->norm_weight || a->ld_out < (int64_t)a->heads * a->vdim) : !a->o) return SLM_ERR_INVALID_ARG;
  if (a->n_single == 0) return SLM_OK;
  SLM_REC_DISPATCH(rec_step)
}
static bool rec_chunks_ok(const slm_recurrent_args& a) {
  return a.pre && a.chunks && a.seq_chunks && a.n_chunks >= 0 && (int64_t)a.n_chunks * a.heads <= 0x7fffffff;
}
extern "C" SLM_API int64_t slm_recurrent_record_floats(int32_t dim_pad, int32_t v_pad) { return 49 * (int64_t)dim_pad + 16 * (int64_t)v_pad + 512; }
extern "C" SLM_API int slm_recurrent_prepare(const slm_recurrent_args* a, void* stream) {
  if (!a || !rec_sizes_ok(*a) || !rec_ptrs_ok(*a) || !rec_chunks_ok(*a)) return SLM_ERR_INVALID_ARG;
  if (!aligned16(a->pre)) return SLM_ERR_ALIGNMENT;
  if (a->n_chunks == 0) return SLM_OK;
  SLM_REC_DISPATCH(rec_prepare)
}
extern "C" SLM_API int slm_recurrent_scan(const slm_recurrent_args* a, void* stream) {
  if (!a || !rec_sizes_ok(*a) || !rec_ptrs_ok(*a) || !rec_chunks_ok(*a) || !a->o) return SLM_ERR_INVALID_ARG;
  if (!aligned16(a->pre)) return SLM_ERR_ALIGNMENT;
  if (a->batch == a->n_single) return SLM_OK;
  SLM_REC_DISPATCH(rec_scan)
}
extern "C" SLM_API int slm_gated_norm(const slm_gated_norm_args* a, void* stream) {
  if (!a || !a->o || !a->gate || !a->weight || !a->out || a->rows < 0 || a->heads < 1 || a->vdim < 1 || a->v_pad < a->vdim || a->v_pad > 256 ||
      a->out_width < (int64_t)a->heads * a->vdim || a->ld_out < a->out_width || a->rows * a->heads > 0x7fffffff)
    return SLM_ERR_INVALID_ARG;
  if (a->dtype != SLM_BF16 && a->dtype != SLM_F32) return SLM_ERR_UNSUPPORTED;
  if (a->rows == 0) return SLM_OK;
  hipStream_t st = (hipStream_t)stream;
  const dim3 grid((unsigned)(a->per_head ? (a->rows * a->heads + 3) / 4 : a->rows)), block(256);
  hip_clear_error();
  if (a->dtype == SLM_BF16) {
    if (a->per_head) gated_norm_kernel<bf16, true><<<grid, block, 0, st>>>(*a);
    else gated_norm_kernel<bf16, false><<<grid, block, 0, st>>>(*a);
  } else {
    if (a->per_head) gated_norm_kernel<float, true><<<grid, block, 0, st>>>(*a);
    else gated_norm_kernel<float, false><<<grid, block, 0, st>>>(*a);
  }
  return hip_check_launch();
}

extern "C" SLM_API const char* slm_mixers_version(void) { return "slm_mixers 1 (gfx950)"; }
extern "C" SLM_API const char* slm_mixers_last_hip_error(void) { return hipGetErrorString((hipError_t)hip_last_error_slot()); }
extern "C" SLM_API const char* slm_mixers_status_string(int s) {
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
