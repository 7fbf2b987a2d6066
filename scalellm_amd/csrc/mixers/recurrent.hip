// recurrent.hip -- layers with a matrix state S [dim, vdim] per sequence and head: the gated delta rule with a decay
// per key channel, and decayed linear attention.  Everything here is fp32 besides the projections it reads.
//
//   step     one row per sequence: convolution, activations, unit vectors, gates, the update and (delta) the output norm
//            in one launch.  One workgroup per (row, head); the state is read and written once.  Bound: HBM (state).
//   prepare  rows of portions: the same inputs, activated and normed, to fp32 buffers.  Bound: HBM.
//   scan     portions: the recurrence, token after token.  The columns of S are independent given q, k, g, so a wave
//            owns 4 CPL of them: lane = (column, row group of 16), the state stays in registers from the portion's first
//            token to its last, both contractions over key channels are register sums and one 16-lane DPP reduction,
//            and no wave waits for another but at the chunks of inputs staged in LDS.  Bound: VALU.
//   gated_norm  the norm and gate behind a scan.
#include "latent/latent_common.h"
#include "slm_mixers.h"

namespace slm {

constexpr bool DELTA_MODE(int m) { return m == SLM_REC_DELTA; }

__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + __expf(-z)); }
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
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
template <typename E>
__device__ __forceinline__ float decay_gate(const slm_recurrent_args& a, int64_t row, int head, int c) {
  const float x = to_f32(reinterpret_cast<const E*>(a.low)[row * a.ld_low + (int64_t)head * a.dim + c]);
  return expf(a.neg_a[head] * softplus_f32(x + a.dt_bias[head * a.dim + c]));
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
        g = decay_gate<E>(a, row, head, i);
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
// prepare: one wave per (portion row, vector): q and k of every q/k head, v of every head, decays of every head
// ---------------------------------------------------------------------------------------
template <typename E, int MODE>
__global__ void __launch_bounds__(256) recurrent_prepare_kernel(const slm_recurrent_args a) {
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int64_t pr = blockIdx.x, row = pr + a.n_single;
  const int s = seq_of_row(a.q_cu, a.batch, (int)row);
  const int64_t row0 = a.q_cu[s];
  const int p = a.positions[row];
  const int n_tasks = 2 * a.qk_heads + (DELTA_MODE(MODE) ? 2 : 1) * a.heads;
  const int qk = a.qk_heads * a.dim;
  const E* ring = nullptr;
  if constexpr (DELTA_MODE(MODE))
    ring = reinterpret_cast<const E*>(a.conv_ring) + (int64_t)a.state_slots[s] * a.taps * (2 * (int64_t)qk + (int64_t)a.heads * a.vdim);
  const E* in = reinterpret_cast<const E*>(a.proj) + row * a.ld_proj;
  for (int task = blockIdx.y * 4 + wave; task < n_tasks; task += 4 * gridDim.y) {
    if (task < 2 * a.qk_heads) {
      const int h = task >> 1, which = task & 1;
      float x[4], ss = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int c = lane + 64 * j;
        x[j] = 0.f;
        if (c < a.dim) {
          if constexpr (DELTA_MODE(MODE)) x[j] = conv_input<E>(a, ring, row, row0, p, which * qk + h * a.dim + c);
          else x[j] = silu_f32(to_f32(in[(which ? a.off_k : a.off_q) + h * a.dim + c]));
        }
        ss = __builtin_fmaf(x[j], x[j], ss);
      }
      float f = 1.0f;
      if constexpr (DELTA_MODE(MODE)) f = (which ? 1.0f : a.q_scale) / sqrtf(wave_sum(ss) + a.unit_eps);
      float* dst = a.pre_qk + ((pr * a.qk_heads + h) * 2 + which) * a.dim_pad;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (lane + 64 * j < a.dim_pad) dst[lane + 64 * j] = x[j] * f;
    } else if (task < 2 * a.qk_heads + a.heads) {
      const int h = task - 2 * a.qk_heads;
      float* dst = a.pre_v + (pr * a.heads + h) * a.v_pad;
      for (int c = lane; c < a.v_pad; c += 64) {
        float v = 0.f;
        if (c < a.vdim) {
          if constexpr (DELTA_MODE(MODE)) v = conv_input<E>(a, ring, row, row0, p, 2 * qk + h * a.vdim + c);
          else v = silu_f32(to_f32(in[a.off_v + h * a.vdim + c]));
        }
        dst[c] = v;
      }
      if constexpr (DELTA_MODE(MODE))
        if (lane == 0) a.pre_beta[pr * a.heads + h] = sigmoid_full(to_f32(in[a.off_b + h]));
    } else if constexpr (DELTA_MODE(MODE)) {
      const int h = task - 2 * a.qk_heads - a.heads;
      float* dst = a.pre_g + (pr * a.heads + h) * a.dim_pad;
      for (int c = lane; c < a.dim_pad; c += 64) dst[c] = c < a.dim ? decay_gate<E>(a, row, h, c) : 1.0f;
    }
  }
}

// ---------------------------------------------------------------------------------------
// scan: workgroup = (sequence, head, 16 CPL columns); DK = 16 R
// ---------------------------------------------------------------------------------------
template <int R>
__device__ __forceinline__ void load_rows(const float* base, int rg, float (&x)[R]) {
  if constexpr (R == 2) {
    const f32x2 t = *reinterpret_cast<const f32x2*>(base + 2 * rg);
    x[0] = t.x, x[1] = t.y;
  } else {
#pragma unroll
    for (int i = 0; i < R / 4; ++i) {
      const f32x4 t = *reinterpret_cast<const f32x4*>(base + 64 * i + 4 * rg);
#pragma unroll
      for (int j = 0; j < 4; ++j) x[4 * i + j] = t[j];
    }
  }
}
template <int R>
__device__ __forceinline__ int row_of(int rg, int r) { return R == 2 ? 2 * rg + r : 64 * (r >> 2) + 4 * rg + (r & 3); }

template <typename E, int MODE, int R, int CPL>
__global__ void __launch_bounds__(256) recurrent_scan_kernel(const slm_recurrent_args a) {
  constexpr bool DELTA = DELTA_MODE(MODE);
  constexpr int DK = 16 * R, NV = DELTA ? 3 : 2, COLS = 16 * CPL;
  constexpr int TC = R > 8 ? 8 : 16;                   // tokens of a staged chunk
  constexpr int ROWF = NV * DK + COLS;                 // floats a token brings: q | k | g | v
  constexpr int V4 = TC * ROWF / 4, PER = (V4 + 255) / 256;
  __shared__ __attribute__((aligned(16))) float buf[2][TC * ROWF];
  __shared__ float sbeta[2][TC];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n_cb = (a.v_pad + COLS - 1) / COLS;
  const int cb = blockIdx.x % n_cb, head = blockIdx.x / n_cb % a.heads, seq = a.n_single + blockIdx.x / (n_cb * a.heads);
  const int64_t row0 = a.q_cu[seq];
  const int n = a.q_cu[seq + 1] - (int)row0;
  const int64_t pr0 = row0 - a.n_single;
  const int p0 = a.positions[row0];
  const int slot = a.state_slots[seq];
  const int qh = head / (a.heads / a.qk_heads);
  const int rg = lane & 15;
  const int col_wg = 4 * CPL * wave + CPL * (lane >> 4);   // first column of this lane in the workgroup
  const int col = cb * COLS + col_wg;
  float* S = a.state + ((int64_t)slot * a.heads + head) * DK * a.v_pad;

  float s[CPL][R];
#pragma unroll
  for (int c = 0; c < CPL; ++c)
#pragma unroll
    for (int r = 0; r < R; ++r) s[c][r] = p0 > 0 && col + c < a.v_pad ? S[(int64_t)row_of<R>(rg, r) * a.v_pad + col + c] : 0.f;

  f32x4 stage[PER];
  float stage_beta = 0.f;
  auto load_chunk = [&](int t0) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int idx = tid + 256 * i, t = idx / (ROWF / 4), e = (idx % (ROWF / 4)) * 4;
      const int64_t pr = pr0 + min(t0 + t, n - 1);
      const float* src;
      if (e < 2 * DK) src = a.pre_qk + (pr * a.qk_heads + qh) * 2 * DK + e;
      else if (DELTA && e < 3 * DK) src = a.pre_g + (pr * a.heads + head) * DK + (e - 2 * DK);
      else src = a.pre_v + (pr * a.heads + head) * a.v_pad + min(cb * COLS + (e - NV * DK), a.v_pad - 4);
      stage[i] = idx < V4 ? *reinterpret_cast<const f32x4*>(src) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
    if (DELTA && tid < TC) stage_beta = a.pre_beta[(pr0 + min(t0 + tid, n - 1)) * a.heads + head];
  };
  auto store_chunk = [&](int b) {
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (tid + 256 * i < V4) *reinterpret_cast<f32x4*>(&buf[b][4 * (tid + 256 * i)]) = stage[i];
    if (DELTA && tid < TC) sbeta[b][tid] = stage_beta;
  };
  const float d = DELTA ? 1.0f : a.decay[head];

  load_chunk(0);
  store_chunk(0);
  __syncthreads();
  for (int t0 = 0, b = 0; t0 < n; t0 += TC, b ^= 1) {
    if (t0 + TC < n) load_chunk(t0 + TC);
    const int m = min(TC, n - t0);
    float keep[CPL];
#pragma unroll
    for (int c = 0; c < CPL; ++c) keep[c] = 0.f;
    auto token = [&](int t) {
      const float* x = &buf[b][t * ROWF];
      float q[R], k[R], v[CPL];
      load_rows<R>(x + DK, rg, k);
#pragma unroll
      for (int c = 0; c < CPL; ++c) v[c] = x[NV * DK + col_wg + c];
      if constexpr (DELTA) {
        float g[R];
        load_rows<R>(x + 2 * DK, rg, g);
        load_rows<R>(x, rg, q);
        const float beta = sbeta[b][t];
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
          float kv[2] = {0.f, 0.f};
#pragma unroll
          for (int r = 0; r < R; ++r) {
            s[c][r] *= g[r];
            kv[r & 1] = __builtin_fmaf(k[r], s[c][r], kv[r & 1]);
          }
          v[c] = beta * (v[c] - group_sum<16>(kv[0] + kv[1]));
        }
      } else {
        load_rows<R>(x, rg, q);
#pragma unroll
        for (int c = 0; c < CPL; ++c)
#pragma unroll
          for (int r = 0; r < R; ++r) s[c][r] *= d;
      }
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        float o[2] = {0.f, 0.f};
#pragma unroll
        for (int r = 0; r < R; ++r) {
          s[c][r] = __builtin_fmaf(k[r], v[c], s[c][r]);
          o[r & 1] = __builtin_fmaf(q[r], s[c][r], o[r & 1]);
        }
        const float sum = group_sum<16>(o[0] + o[1]);
        keep[c] = rg == t ? sum : keep[c];
      }
    };
    if (m == TC) {
#pragma unroll 4
      for (int t = 0; t < TC; ++t) token(t);
    } else {
      for (int t = 0; t < m; ++t) token(t);
    }
    if (rg < m)
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        if (col + c < a.v_pad) a.o[((pr0 + t0 + rg) * a.heads + head) * a.v_pad + col + c] = keep[c];
    if (t0 + TC < n) store_chunk(b ^ 1);
    __syncthreads();
  }
#pragma unroll
  for (int c = 0; c < CPL; ++c)
    if (col + c < a.v_pad)
#pragma unroll
      for (int r = 0; r < R; ++r) S[(int64_t)row_of<R>(rg, r) * a.v_pad + col + c] = s[c][r];

  // the last inputs of the convolutions (their readers ran in the launch before)
  if (DELTA && cb == 0) {
    const int qk = a.qk_heads * a.dim;
    const int64_t ch = 2 * (int64_t)qk + (int64_t)a.heads * a.vdim;
    E* ring = reinterpret_cast<E*>(a.conv_ring) + (int64_t)slot * a.taps * ch;
    const bool first_of_group = head % (a.heads / a.qk_heads) == 0;
    for (int j = max(0, n - a.taps); j < n; ++j) {
      E* dst = ring + (int64_t)((p0 + j) % a.taps) * ch;
      if (first_of_group)
        for (int i = tid; i < a.dim; i += 256) {
          dst[qh * a.dim + i] = raw_input<E>(a, row0 + j, qh * a.dim + i);
          dst[qk + qh * a.dim + i] = raw_input<E>(a, row0 + j, qk + qh * a.dim + i);
        }
      for (int i = tid; i < a.vdim; i += 256) dst[2 * qk + head * a.vdim + i] = raw_input<E>(a, row0 + j, 2 * qk + head * a.vdim + i);
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
    float ss = 0.f;
    for (int c = lane; c < a.vdim; c += 64) ss = __builtin_fmaf(o[c], o[c], ss);
    const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
    const E* gate = reinterpret_cast<const E*>(a.gate) + row * a.ld_gate + (int64_t)h * a.vdim;
    E* out = reinterpret_cast<E*>(a.out) + row * a.ld_out;
    for (int c = lane; c < a.vdim; c += 64)
      out[h * a.vdim + c] = (E)(a.scale * o[c] * rs * a.weight[c] * sigmoid_f32(to_f32(gate[c])));
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
template <typename E, int MODE, int R>
static void rec_scan_r(const slm_recurrent_args& a, hipStream_t st) {
  const int64_t items = (int64_t)(a.batch - a.n_single) * a.heads;
  // two columns per lane read the staged rows half as often: where enough workgroups are left to fill the chip
  if (R <= 8 && items * ((a.v_pad + 31) / 32) >= 512)
    recurrent_scan_kernel<E, MODE, R, (R <= 8 ? 2 : 1)><<<dim3((unsigned)(items * ((a.v_pad + 31) / 32))), dim3(256), 0, st>>>(a);
  else
    recurrent_scan_kernel<E, MODE, R, 1><<<dim3((unsigned)(items * ((a.v_pad + 15) / 16))), dim3(256), 0, st>>>(a);
}
template <typename E, int MODE>
static int rec_scan(const slm_recurrent_args& a, hipStream_t st) {
  hip_clear_error();
  switch (a.dim_pad / 16) {
    case 2: rec_scan_r<E, MODE, 2>(a, st); break;
    case 4: rec_scan_r<E, MODE, 4>(a, st); break;
    case 8: rec_scan_r<E, MODE, 8>(a, st); break;
    case 12: rec_scan_r<E, MODE, 12>(a, st); break;
    default: rec_scan_r<E, MODE, 16>(a, st);
  }
  return hip_check_launch();
}
template <typename E, int MODE>
static int rec_prepare(const slm_recurrent_args& a, hipStream_t st) {
  const int n_tasks = 2 * a.qk_heads + (MODE == SLM_REC_DELTA ? 2 : 1) * a.heads;
  hip_clear_error();
  recurrent_prepare_kernel<E, MODE><<<dim3((unsigned)(a.rows - a.n_single), (unsigned)((n_tasks + 3) / 4)), dim3(256), 0, st>>>(a);
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
extern "C" SLM_API int slm_recurrent_prepare(const slm_recurrent_args* a, void* stream) {
  if (!a || !rec_sizes_ok(*a) || !rec_ptrs_ok(*a) || !a->pre_qk || !a->pre_v) return SLM_ERR_INVALID_ARG;
  if (a->mode == SLM_REC_DELTA && (!a->pre_g || !a->pre_beta)) return SLM_ERR_INVALID_ARG;
  if (a->rows == a->n_single) return SLM_OK;
  SLM_REC_DISPATCH(rec_prepare)
}
extern "C" SLM_API int slm_recurrent_scan(const slm_recurrent_args* a, void* stream) {
  if (!a || !rec_sizes_ok(*a) || !rec_ptrs_ok(*a) || !a->pre_qk || !a->pre_v || !a->o) return SLM_ERR_INVALID_ARG;
  if (a->mode == SLM_REC_DELTA && (!a->pre_g || !a->pre_beta)) return SLM_ERR_INVALID_ARG;
  if (!aligned16(a->pre_qk) || !aligned16(a->pre_v) || !aligned16(a->pre_g)) return SLM_ERR_ALIGNMENT;
  if (a->batch == a->n_single) return SLM_OK;
  SLM_REC_DISPATCH(rec_scan)
}
extern "C" SLM_API int slm_gated_norm(const slm_gated_norm_args* a, void* stream) {
  if (!a || !a->o || !a->gate || !a->weight || !a->out || a->rows < 0 || a->heads < 1 || a->vdim < 1 || a->v_pad < a->vdim ||
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
