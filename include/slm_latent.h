/*
 * slm_latent.h -- C ABI of libslm_latent.so: the MI355X (gfx950) kernels of the dense 16-/32-bit model
 * path (residual stream, norms, products) and of latent attention (scalellm_amd/dagupel.py).  The mechanisms
 * are separate entry points with their constants as arguments.
 *
 * Conventions are those of slm_hip.h: plain pointers and sizes, asynchronous on `stream`, nothing is
 * allocated or synchronised (hipGraph-capturable), 0 or a negative slm_status comes back.
 *
 * dtype: SLM_BF16 or SLM_F32 -- the type of weights, activations and cache.  The residual stream, norms,
 * rotation angles, attention scores and soft-max weights and split partials are fp32 in either case.
 */
#ifndef SLM_LATENT_H_
#define SLM_LATENT_H_

#include "slm_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

#define SLM_F32 2

SLM_API const char* slm_latent_version(void);
SLM_API const char* slm_latent_status_string(int status);
SLM_API const char* slm_latent_last_hip_error(void);

/* ---- 1. fp32 residual stream: (embedding | add) + norm -------------------------------------------- */
/* norms: RMS x / sqrt(mean x^2 + eps) * weight;  TANH tanh(alpha x) * weight + bias                    */
typedef struct slm_residual_norm_args {
  float* resid;             /* [rows, width] fp32, read and written (written only by EMBED)             */
  const void* delta;        /* ADD: [rows, width] of dtype, row stride ld_delta                         */
  const float* slabs;       /* SLABS: [n_slabs][rows][ld_delta] fp32 split-K partial sums               */
  const int32_t* tokens;    /* EMBED: [rows]                                                            */
  const int32_t* positions; /* EMBED with a position table: [rows]                                      */
  const void* embed;        /* EMBED: [vocab, ld_embed] of dtype                                        */
  const void* pos_table;    /* EMBED: [max_positions, width] of dtype, or NULL                          */
  const int32_t* row_index; /* NULL, or [rows]: output row r is made of stream row row_index[r] (PLAIN) */
  const float* weight;      /* [width] fp32; NULL: only the sum, no norm                                */
  const float* bias;        /* TANH: [width] fp32                                                       */
  void* out;                /* [rows, ld_out] of dtype; columns width .. ld_out-1 are zeroed            */
  int64_t rows, width, ld_delta, ld_embed, ld_out, slab_stride;
  float eps, norm_alpha;
  float delta_mult;         /* factor of what is added: the delta, or the embedding row                 */
  int32_t n_slabs, mode, dtype, norm;
} slm_residual_norm_args;
enum { SLM_NORM_RMS = 0, SLM_NORM_TANH = 1 };
enum { SLM_RN_EMBED = 0, SLM_RN_ADD = 1, SLM_RN_SLABS = 2, SLM_RN_PLAIN = 3 };
SLM_API int slm_residual_norm(const slm_residual_norm_args* a, void* stream);

/* ---- 2. y = x W^T by one wave-tile kernel (MFMA 16x16), weights streamed -------------------------- */
/* x [batch][M, K], w [batch][N, K] (K contiguous, K % 64 == 0, N % 16 == 0).  Epilogues:               */
/*   STORE   y[m, n] of dtype;  F32  y[m, n] = alpha * acc as fp32;                                     */
/*   SLABS   y = fp32 [n_splits][M][ldy] partial sums (the consumer adds them, slm_residual_norm);      */
/*   GLU     w = [gate | up] (N = 2 * half): y[m, n] = glu(gate, up) as below, width half;              */
/*   GATE    y = acc * sigmoid(gate[m * ld_gate + batch index]) (per-head output gate).                 */
typedef struct slm_linear_args {
  const void* x; const void* w; void* y; const void* gate;
  int64_t M, N, K, ldx, ldw, ldy, ld_gate;
  int64_t x_batch, w_batch, y_batch;   /* element strides between batch items                           */
  float alpha, limit, glu_alpha, glu_shift;
  int32_t batch, n_splits, epilogue, dtype;
} slm_linear_args;
enum { SLM_LIN_STORE = 0, SLM_LIN_F32 = 1, SLM_LIN_SLABS = 2, SLM_LIN_GLU = 3, SLM_LIN_GATE = 4 };
SLM_API int slm_linear(const slm_linear_args* a, void* stream);
/* y = g sigmoid(alpha g) (u + shift), g = min(gate, limit), u = clamp(up, +-limit) (limit may be        */
/* infinite: with alpha 1 and shift 0 the plain SiLU GLU); gu = [rows, 2 * half]                         */
SLM_API int slm_clamped_glu(void* y, const void* gu, int64_t rows, int64_t half, int64_t ld_gu, int64_t ld_y,
                            float limit, float glu_alpha, float glu_shift, int32_t dtype, void* stream);

/* ---- 3. latent cache append: latent RMS norm, rotation of the shared key part and of the queries --- */
typedef struct slm_latent_append_args {
  void* proj;               /* [rows, ld_proj]: q heads at 0 ([heads][q_dim | q_rot]), latent at off_c,
                             * rotated key part at off_r; the q_rot parts are rotated in place            */
  void* cache;              /* [slots, c_pad + r_pad]: normed latent | rotated key part, zero padded      */
  void* q_abs;              /* [abs_rows, heads, c_pad + r_pad] or NULL: rotated q copied behind c_pad    */
  const float* norm_weight; /* [rank]                                                                     */
  const float* cos_sin;     /* [max_positions, rot] = cos | sin (magnitude folded in)                     */
  const int32_t* positions; /* [rows] */
  const int32_t* slots;     /* [rows] */
  int64_t rows, abs_rows, ld_proj, off_c, off_r, max_positions;
  int32_t heads, q_dim, q_rot, rank, rot, c_pad, r_pad, dtype;
  float eps;
} slm_latent_append_args;
SLM_API int slm_latent_append(const slm_latent_append_args* a, void* stream);

/* ---- 4. attention over the paged latent cache (absorbed queries), one work item per query row ----- */
/* scores q_abs . row * scale over positions [max(0, p - window + 1), p]; out = soft-max weighted latent */
typedef struct slm_latent_attn_args {
  const void* q_abs;        /* [rows, heads, c_pad + r_pad]  */
  const void* cache;        /* [slots, c_pad + r_pad]        */
  void* out;                /* [rows, heads, c_pad]          */
  const int32_t* positions; /* [rows]                        */
  const int32_t* q_cu;      /* [batch + 1]: row -> sequence  */
  const int32_t* block_table; const int32_t* block_cu;
  void* workspace; size_t workspace_bytes;
  int64_t rows;
  int32_t batch, heads, c_pad, r_pad, block_size, window /* <= 0: none */, max_kv_len /* hint */, n_splits /* 0 = auto */;
  float scale;
  int32_t dtype;
  int32_t generic;          /* 1 = the any-size kernel (tests)   */
} slm_latent_attn_args;
SLM_API size_t slm_latent_attn_workspace_bytes(const slm_latent_attn_args* a);
SLM_API int slm_latent_attn(const slm_latent_attn_args* a, void* stream);
/* 1 if the MFMA kernel serves these sizes, 0: the any-size kernel */
SLM_API int slm_latent_attn_is_mfma(int32_t c_pad, int32_t r_pad, int32_t dtype);

/* ---- 5. prompt portions: gather latent rows, attention over expanded keys and values --------------- */
SLM_API int slm_latent_gather(void* out /* [n, row] */, const void* cache, const int32_t* slots, int64_t n,
                              int64_t row_bytes, void* stream);
typedef struct slm_latent_prefill_args {
  const void* q;            /* rows of proj, q heads at column 0: [heads][q_dim + r_pad]                 */
  const void* ctx;          /* [n_ctx, c_pad + r_pad] gathered latent rows (the rotated key parts)       */
  const void* kv;           /* [n_ctx, heads * (q_dim + v_pad)]: unrotated key | value per head          */
  const void* gate;         /* logits of the output gate, [row * ld_q + gate_off + head] of q's buffer   */
  void* out;                /* [rows, ld_out]: [heads][v_pad]                                            */
  const int32_t* tiles;     /* [n_tiles][6]: first row, rows, ctx base, ctx length, first ctx position,
                             * position of the first row                                                 */
  int64_t ld_q, ld_out, n_rows, n_ctx, gate_off;
  int32_t n_tiles, heads, q_dim, c_pad, r_pad, v_pad, window;
  float scale;
} slm_latent_prefill_args;
SLM_API int slm_latent_prefill(const slm_latent_prefill_args* a, void* stream);
SLM_API int slm_latent_prefill_supported(int32_t q_dim, int32_t r_pad, int32_t v_pad);
#define SLM_LATENT_Q_TILE 128

#ifdef __cplusplus
}
#endif
#endif
