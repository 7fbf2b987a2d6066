// window_attn.hip -- paged grouped-query attention with a window, kept first tokens, capped scores and a sink: the cache
// append, and the any-size attention kernel (32-bit; widths the MFMA kernels do not have).
#include "window_common.h"

namespace slm {

constexpr int WA_MAX = 512;   // widest head

// one wave per (row, vector): q heads normed and rotated in place, k heads normed and rotated into the cache, v copied
template <typename E, int NJ>   // NJ: columns per lane
__global__ void __launch_bounds__(256) window_append_kernel(const slm_window_append_args a) {
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int64_t row = blockIdx.x;
  const int task = blockIdx.y * 4 + wave;
  if (task >= a.heads + 2 * a.kv_heads) return;
  E* pr = reinterpret_cast<E*>(a.proj) + row * a.ld_proj;
  const int64_t slot = a.slots[row];
  if (task >= a.heads + a.kv_heads) {
    const int g = task - a.heads - a.kv_heads;
    const E* src = pr + a.off_v + (int64_t)g * a.v_pad;
    E* dst = reinterpret_cast<E*>(a.value_cache) + (slot * a.kv_heads + g) * a.v_pad;
    for (int c = lane; c < a.v_pad; c += 64) dst[c] = src[c];
    return;
  }
  const bool is_q = task < a.heads;
  const int g = is_q ? task : task - a.heads;
  E* src = pr + (is_q ? a.off_q : a.off_k) + (int64_t)g * a.d_pad;
  const float* w = is_q ? a.q_weight : a.k_weight;
  const int64_t p = min((int64_t)a.positions[row], a.max_positions - 1);
  const float* cs = a.cos_sin + p * a.rot;
  const int half = a.rot / 2;
  float x[NJ], y[NJ], ss = 0.f;
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int c = lane + 64 * j;
    x[j] = y[j] = 0.f;
    if (c < a.dim) {
      x[j] = to_f32(src[c]);
      ss = __builtin_fmaf(x[j], x[j], ss);
      if (c < a.rot) {
        const int o = c < half ? c + half : c - half;
        y[j] = to_f32(src[o]) * w[o];
      }
      x[j] *= w[c];
    }
  }
  const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
  E* dst = is_q ? src : reinterpret_cast<E*>(a.key_cache) + (slot * a.kv_heads + g) * a.d_pad;
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int c = lane + 64 * j;
    if (c >= a.d_pad) continue;
    float v = x[j] * rs;
    if (c < a.rot) {
      const float co = cs[c < half ? c : c - half], si = cs[half + (c < half ? c : c - half)];
      v = c < half ? v * co - y[j] * rs * si : v * co + y[j] * rs * si;
    }
    dst[c] = (E)v;
  }
}

// One workgroup per (row, head); a wave takes tiles of 64 keys: lane = key for the scores, lane = column for the sums.
template <typename E>
__global__ void __launch_bounds__(256) window_attn_any_kernel(const slm_window_attn_args a) {
  __shared__ float sq[WA_MAX], sp[4][64], sm[4], sl[4], so[4][WA_MAX];
  __shared__ int64_t ss[4][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int head = blockIdx.x % a.heads;
  const int64_t row = blockIdx.x / a.heads;
  const int g = head / (a.heads / a.kv_heads);
  const int seq = seq_of_row(a.q_cu, a.batch, (int)row);
  const int32_t* table = a.block_table + a.block_cu[seq];
  const VisibleKeys vis(a.positions[row], a.window, a.keep_first);
  const E* q = reinterpret_cast<const E*>(a.q) + row * a.ld_q + (int64_t)head * a.d_pad;
  for (int i = tid; i < a.d_pad; i += 256) sq[i] = to_f32(q[i]);
  __syncthreads();
  const E* kc = reinterpret_cast<const E*>(a.key_cache) + (int64_t)g * a.d_pad;
  const E* vc = reinterpret_cast<const E*>(a.value_cache) + (int64_t)g * a.v_pad;
  float m = M_INIT_F, l = 0.f, o[WA_MAX / 64];
#pragma unroll
  for (int j = 0; j < WA_MAX / 64; ++j) o[j] = 0.f;
  for (int i0 = 64 * wave; i0 < vis.count; i0 += 256) {
    const int n = min(64, vis.count - i0);
    const int pos = vis.position(i0 + min(lane, n - 1));
    const int64_t slot = table[pos / a.block_size] + pos % a.block_size;
    const E* k = kc + slot * a.kv_heads * a.d_pad;
    float s = 0.f;
    for (int c = 0; c < a.d_pad; c += 4) {
      float t[4];
      load_f32<4>(k + c, t);
#pragma unroll
      for (int j = 0; j < 4; ++j) s = __builtin_fmaf(t[j], sq[c + j], s);
    }
    s *= a.scale;
    if (a.softcap > 0.f) s = a.softcap * tanhf(s / a.softcap);
    if (lane >= n) s = -INFINITY;
    const float m_new = fmaxf(m, wave_max(s));
    const float f = expf(m - m_new), e = expf(s - m_new);
    m = m_new;
    l = l * f + wave_sum(e);
    sp[wave][lane] = e;
    ss[wave][lane] = slot;
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int j = 0; j < WA_MAX / 64; ++j) o[j] *= f;
    for (int t = 0; t < n; ++t) {
      const float e_t = sp[wave][t];
      const E* v = vc + ss[wave][t] * a.kv_heads * a.v_pad;
#pragma unroll
      for (int j = 0; j < WA_MAX / 64; ++j)
        if (lane + 64 * j < a.v_pad) o[j] = __builtin_fmaf(e_t, to_f32(v[lane + 64 * j]), o[j]);
    }
    __builtin_amdgcn_wave_barrier();
  }
  if (lane == 0) sm[wave] = m, sl[wave] = l;
#pragma unroll
  for (int j = 0; j < WA_MAX / 64; ++j)
    if (lane + 64 * j < a.v_pad) so[wave][lane + 64 * j] = o[j];
  __syncthreads();
  float top = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
  if (a.sink) top = fmaxf(top, a.sink[head]);
  float f[4], total = a.sink ? expf(a.sink[head] - top) : 0.f;
#pragma unroll
  for (int w = 0; w < 4; ++w) {
    f[w] = expf(sm[w] - top);
    total += f[w] * sl[w];
  }
  E* out = reinterpret_cast<E*>(a.out) + row * a.ld_out + (int64_t)head * a.v_pad;
  for (int c = tid; c < a.v_pad; c += 256) {
    float x = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) x = __builtin_fmaf(f[w], so[w][c], x);
    out[c] = (E)(a.out_scale * x / total);
  }
}

template <typename E>
static void append_launch(const slm_window_append_args& a, dim3 grid, hipStream_t st) {
  switch ((a.d_pad + 63) / 64) {
    case 1: window_append_kernel<E, 1><<<grid, dim3(256), 0, st>>>(a); break;
    case 2: window_append_kernel<E, 2><<<grid, dim3(256), 0, st>>>(a); break;
    case 3: case 4: window_append_kernel<E, 4><<<grid, dim3(256), 0, st>>>(a); break;
    default: window_append_kernel<E, WA_MAX / 64><<<grid, dim3(256), 0, st>>>(a);
  }
}

bool window_decode_ok(const slm_window_attn_args& a);
size_t window_decode_workspace(const slm_window_attn_args& a);
int window_decode(const slm_window_attn_args& a, hipStream_t st);

}  // namespace slm

using namespace slm;

extern "C" SLM_API int slm_window_append(const slm_window_append_args* a, void* stream) {
  if (!a || !a->proj || !a->key_cache || !a->value_cache || !a->q_weight || !a->k_weight || !a->positions || !a->slots ||
      a->rows < 0 || a->heads < 1 || a->kv_heads < 1 || a->heads % a->kv_heads || a->dim < 1 || a->dim > a->d_pad || a->rot < 0 ||
      a->rot % 2 || a->rot > a->dim || (a->rot && (!a->cos_sin || a->max_positions < 1)))
    return SLM_ERR_INVALID_ARG;
  if (a->d_pad > WA_MAX || (a->dtype != SLM_BF16 && a->dtype != SLM_F32)) return SLM_ERR_UNSUPPORTED;
  if (a->rows == 0) return SLM_OK;
  const dim3 grid((unsigned)a->rows, (unsigned)((a->heads + 2 * a->kv_heads + 3) / 4));
  hip_clear_error();
  if (a->dtype == SLM_BF16) append_launch<bf16>(*a, grid, (hipStream_t)stream);
  else append_launch<float>(*a, grid, (hipStream_t)stream);
  return hip_check_launch();
}

static bool wa_ok(const slm_window_attn_args* a) {
  return a && a->q && a->key_cache && a->value_cache && a->out && a->positions && a->q_cu && a->block_table && a->block_cu &&
         a->rows >= 0 && a->batch >= 1 && a->heads >= 1 && a->kv_heads >= 1 && a->heads % a->kv_heads == 0 && a->d_pad > 0 &&
         a->v_pad > 0 && a->block_size > 0 && a->rows * a->heads <= 0x7fffffff;
}
extern "C" SLM_API size_t slm_window_attn_workspace_bytes(const slm_window_attn_args* a) {
  if (!wa_ok(a) || a->generic || !window_decode_ok(*a)) return 0;
  return window_decode_workspace(*a);
}
extern "C" SLM_API int slm_window_attn(const slm_window_attn_args* a, void* stream) {
  if (!wa_ok(a)) return SLM_ERR_INVALID_ARG;
  if (a->d_pad > WA_MAX || a->v_pad > WA_MAX || a->d_pad % 8 || a->v_pad % 8 || (a->dtype != SLM_BF16 && a->dtype != SLM_F32))
    return SLM_ERR_UNSUPPORTED;
  if (a->ld_q % 8 || a->ld_out % 4 || !aligned16(a->q) || !aligned16(a->key_cache) || !aligned16(a->value_cache))
    return SLM_ERR_ALIGNMENT;
  if (a->rows == 0) return SLM_OK;
  if (!a->generic && window_decode_ok(*a)) return window_decode(*a, (hipStream_t)stream);
  const dim3 grid((unsigned)(a->rows * a->heads));
  hip_clear_error();
  if (a->dtype == SLM_BF16) window_attn_any_kernel<bf16><<<grid, dim3(256), 0, (hipStream_t)stream>>>(*a);
  else window_attn_any_kernel<float><<<grid, dim3(256), 0, (hipStream_t)stream>>>(*a);
  return hip_check_launch();
}
