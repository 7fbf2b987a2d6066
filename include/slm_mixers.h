/*
 * slm_mixers.h -- C ABI of libslm_mixers.so: the MI355X (gfx950) kernels of two families of token mixers beside the
 * dense path of slm_latent.h: paged grouped-query attention with a window, kept first tokens, capped scores and a sink,
 * and recurrent layers with a matrix state per head (gated delta rule, decayed linear attention).  Constants of a
 * design are arguments.
 *
 * Conventions are those of slm_hip.h: plain pointers and sizes, asynchronous on `stream`, nothing is allocated or
 * synchronised (hipGraph-capturable), 0 or a negative slm_status comes back.
 *
 * dtype: SLM_BF16 or SLM_F32 -- weights, activations, key / value cache.  Norms, rotation, scores, soft-max weights'
 * sums, recurrent state and everything that enters a recurrence besides projections are fp32 in either case.
 */
#ifndef SLM_MIXERS_H_
#define SLM_MIXERS_H_

#include "slm_latent.h"

#ifdef __cplusplus
extern "C" {
#endif

SLM_API const char* slm_mixers_version(void);
SLM_API const char* slm_mixers_status_string(int status);
SLM_API const char* slm_mixers_last_hip_error(void);

/* ---- 1. recurrent layers: state S [dim, vdim] per sequence and head -------------------------------- */
/*   DELTA      S <- g S (g per key channel);  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q          */
/*              q, k, v: short causal convolution + silu; q, k unit vectors, q scaled;                    */
/*              g = exp(neg_a softplus(low + dt_bias)), beta = sigmoid                                     */
/*   LIGHTNING  S <- decay S + k v^T;  o = S^T q;  q, k, v: silu                                           */
/* A batch is sequences of rows q_cu[s] .. q_cu[s + 1]; the first n_single sequences bring one row each    */
/* (slm_recurrent_step), the others go through prepare + scan.  A row at position 0 starts from a zero     */
/* state, whatever its slot holds.                                                                         */
enum { SLM_REC_DELTA = 0, SLM_REC_LIGHTNING = 1 };
typedef struct slm_recurrent_args {
  const void* proj;          /* [rows, ld_proj] of dtype: q [qk_heads][dim], k, v [heads][vdim] at off_*, beta
                              * logits [heads] at off_b (DELTA)                                             */
  const void* low;           /* DELTA: [rows, ld_low] of dtype: decay inputs [heads][dim] at 0, gate logits
                              * [heads][vdim] at off_gate                                                   */
  const float* conv_w;       /* DELTA: [taps][conv_channels], last tap = the current token; channels q | k | v */
  void* conv_ring;           /* DELTA: [slots][taps][conv_channels] of dtype, the input of position p at p % taps */
  float* state;              /* [slots][heads][dim_pad][v_pad]                                              */
  const float* neg_a;        /* DELTA: [heads] = -exp(A_log)                                                */
  const float* dt_bias;      /* DELTA: [heads][dim]                                                         */
  const float* decay;        /* LIGHTNING: [heads]                                                          */
  const float* norm_weight;  /* DELTA: [vdim] (slm_recurrent_step applies norm and gate itself)             */
  const int32_t* positions;  /* [rows]                                                                      */
  const int32_t* q_cu;       /* [batch + 1]                                                                 */
  const int32_t* state_slots;/* [batch]                                                                     */
  const int32_t* chunks;     /* prepare: [n_chunks][3]: sequence, first row, rows (<= 16) of every portion's chunks */
  const int32_t* seq_chunks; /* scan: [batch - n_single]: a portion's first chunk (its chunks follow each other) */
  float* pre;                /* prepare -> scan: [n_chunks][heads] records of slm_recurrent_record_floats   */
  float* o;                  /* scan: [portion rows][heads][v_pad]; step, LIGHTNING: [n_single][heads][v_pad] */
  void* out;                 /* step, DELTA: [n_single, ld_out] of dtype, [heads][vdim], zero padded to ld_out */
  int64_t rows, ld_proj, ld_low, ld_out, off_q, off_k, off_v, off_b, off_gate;
  int32_t mode, dtype, batch, n_single, n_slots, heads, qk_heads, dim, vdim, dim_pad, v_pad, taps, n_chunks;
  float q_scale, eps, unit_eps;
} slm_recurrent_args;
/* the padded key width of the state for `dim` (0: not served), v_pad = vdim rounded up to 16 (at most 256) */
SLM_API int32_t slm_recurrent_dim_pad(int32_t dim);
SLM_API int64_t slm_recurrent_record_floats(int32_t dim_pad, int32_t v_pad);
SLM_API int slm_recurrent_step(const slm_recurrent_args* a, void* stream);
SLM_API int slm_recurrent_prepare(const slm_recurrent_args* a, void* stream);
SLM_API int slm_recurrent_scan(const slm_recurrent_args* a, void* stream);

/* ---- 2. y = scale * rms_norm(o over a group) * weight * sigmoid(gate) -------------------------------- */
/* group = one head (per_head: weight [vdim]) or all heads together (weight [heads * vdim])               */
typedef struct slm_gated_norm_args {
  const float* o;        /* [rows][heads][v_pad]                                                           */
  const void* gate;      /* [rows, ld_gate] of dtype, [heads][vdim]                                        */
  const float* weight;
  void* out;             /* [rows, ld_out] of dtype, [heads][vdim]; columns up to out_width are zeroed     */
  int64_t rows, ld_gate, ld_out, out_width;
  int32_t heads, vdim, v_pad, per_head, dtype;
  float eps, scale;
} slm_gated_norm_args;
SLM_API int slm_gated_norm(const slm_gated_norm_args* a, void* stream);

/* ---- 3. windowed attention: append --------------------------------------------------------------------- */
/* RMS norm per head, rotation of the first `rot` dimensions (pairs i, i + rot / 2), key / value -> cache;   */
/* queries in place.  Heads are d_pad / v_pad wide, zero padded                                              */
typedef struct slm_window_append_args {
  void* proj;                /* [rows, ld_proj]: q [heads][d_pad], k [kv_heads][d_pad], v [kv_heads][v_pad] at off_* */
  void* key_cache;           /* [slots][kv_heads][d_pad] */
  void* value_cache;         /* [slots][kv_heads][v_pad] */
  const float* q_weight; const float* k_weight;   /* [dim] */
  const float* cos_sin;      /* [max_positions, rot] = cos | sin */
  const int32_t* positions; const int32_t* slots; /* [rows] */
  int64_t rows, ld_proj, off_q, off_k, off_v, max_positions, n_slots;
  int32_t heads, kv_heads, dim, rot, d_pad, v_pad, dtype;
  float eps;
} slm_window_append_args;
SLM_API int slm_window_append(const slm_window_append_args* a, void* stream);

/* ---- 4. windowed attention over the paged cache, one work item per query row ----------------------------- */
/* position i sees j <= i with i - j < window (window <= 0: all) or j < keep_first; score = q.k * scale, then
 * softcap * tanh(score / softcap) (softcap <= 0: none); the denominator also holds exp(sink[head]);
 * out = out_scale * result                                                                                  */
typedef struct slm_window_attn_args {
  const void* q;             /* [rows, ld_q]: [heads][d_pad] */
  const void* key_cache; const void* value_cache;
  void* out;                 /* [rows, ld_out]: [heads][v_pad] */
  const float* sink;         /* [heads] or NULL */
  const int32_t* positions; const int32_t* q_cu; const int32_t* block_table; const int32_t* block_cu;
  void* workspace; size_t workspace_bytes;
  int64_t rows, ld_q, ld_out;
  int32_t batch, heads, kv_heads, d_pad, v_pad, block_size, window, keep_first, max_kv_len /* hint */, n_splits /* 0 = auto */;
  float scale, softcap, out_scale;
  int32_t dtype, generic /* 1 = the any-size kernel (tests) */;
} slm_window_attn_args;
SLM_API size_t slm_window_attn_workspace_bytes(const slm_window_attn_args* a);
SLM_API int slm_window_attn(const slm_window_attn_args* a, void* stream);

/* ---- 5. the same for prompt portions (bf16, MFMA) ---------------------------------------------------------- */
/* A portion's context is a list of cache slots: its kept first positions 0 .. n_kept - 1, then every position
 * from `first` (>= n_kept) on.                                                                                 */
typedef struct slm_window_prefill_args {
  const void* q;
  const void* key_cache; const void* value_cache;
  void* out;
  const float* sink;
  const int32_t* slots;      /* [n_ctx] */
  const int32_t* tiles;      /* [n_tiles][7]: first row, rows, ctx base, ctx length, kept, first, position of the first row */
  int64_t ld_q, ld_out, n_rows, n_ctx;
  int32_t n_tiles, heads, kv_heads, d_pad, v_pad, window, keep_first;
  float scale, softcap, out_scale;
} slm_window_prefill_args;
SLM_API int slm_window_prefill(const slm_window_prefill_args* a, void* stream);
SLM_API int slm_window_prefill_supported(int32_t d_pad, int32_t v_pad);
#define SLM_WINDOW_Q_TILE 128

#ifdef __cplusplus
}
#endif
#endif
