/*
 * astrai_seq -- C ABI of the kernels for decoders that mix linear recurrences with
 * sliding-window attention (libastrai_seq.so, gfx950).
 *
 * Conventions as in astrai_q.h: device pointers owned by the caller, no allocation, no
 * synchronisation, work queued on `stream`, AQ_* return codes and dtype codes.  `dtype`
 * is the element type of activations, weights and caches (the void pointers); float
 * pointers are fp32 whatever it is.
 *
 * M = B * S rows: B sequences with S new tokens each.  Per-sequence inputs in device
 * memory: pos[b] the position of the first new token, slots[b] the sequence's place in
 * the state tensors.  A sequence at position 0 starts from empty state, whatever its
 * slot holds.  ld*: elements between consecutive rows; o_*: first column of a part
 * inside the fused projection's row.
 */
#ifndef ASTRAI_SEQ_H
#define ASTRAI_SEQ_H

#include "astrai_q.h"

#ifdef __cplusplus
extern "C" {
#endif

/* ---- rows */
/* x[m] = table[ids[m]] (fp32; an id outside the table gives a zero row). */
int aqs_embed(const int64_t *ids, const void *table, int dtype, float *x, int64_t M, int64_t K, int64_t V, void *stream);
/* x += mult * y (y may be NULL); out = x / sqrt(mean(x^2) + eps) * (1 + w) (out may be NULL when y is given). */
int aqs_add_rmsnorm(float *x, const void *y, int64_t ldy, int dtype, float mult, const float *w, float eps, void *out,
                    int64_t M, int64_t K, void *stream);
/* gu [M, 2F] = gate | up;  g = min(gate, limit), u = clamp(up, -limit, limit);  out = g sigmoid(1.702 g) (u + 1). */
int aqs_clamped_glu(const void *gu, int64_t ld, int dtype, float limit, void *out, int64_t M, int64_t F, void *stream);
/* out = RMS over each of `groups` equal parts of y * silu(z), times w [K]. */
int aqs_gated_group_norm(const float *y, const void *z, int64_t ldz, int dtype, const float *w, float eps, void *out,
                         int64_t ldo, int64_t M, int64_t K, int64_t groups, void *stream);
/* Per head of o [M, H, E]: RMS over E, times w [E], times sigmoid(gate [M, H*E]), times scale. */
int aqs_head_norm_gate(const float *o, const void *gate, int64_t ldg, int dtype, const float *w, float eps, float scale,
                       void *out, int64_t ldo, int64_t M, int64_t H, int64_t E, void *stream);

/* ---- matrix-vector products of a decode step (w [N, K] of dtype)
 * in_kind  0: x of dtype [M, ldx]   1: RMSNorm of xf [M, K] with gain around zero
 *          2: gated group norm of xf [M, K] with z = x (stride ldx), gain [K], groups
 * out_kind 0: out of dtype (+ bias) 1: fp32 into res   2: res += mult * result
 *          3: clamped GLU of w's first N/2 rows (gate) and last N/2 rows (up), out [M, N/2]
 * Pairs served: 0-0, 0-2, 1-0, 1-1, 1-3, 2-2; sizes: aqs_gemv_ok. */
int aqs_gemv_ok(int dtype, int64_t M, int64_t N, int64_t K);
int aqs_gemv(int in_kind, int out_kind, int dtype, const void *x, int64_t ldx, const float *xf, const float *gain, float eps,
             int64_t groups, const void *w, const float *bias, float mult, float limit, float *res, void *out, int64_t ldo,
             int64_t M, int64_t N, int64_t K, void *stream);

/* ---- causal per-channel convolution; ring [slots, taps, C]: the input of position p in place p % taps */
int aqs_conv_silu(const void *in, int64_t ld, int dtype, const float *w, const float *bias, const void *ring,
                  const int32_t *slots, const int32_t *pos, float *out, int64_t B, int64_t S, int64_t C, int64_t taps,
                  void *stream);
/* The last taps - 1 of the S new inputs go into the ring (after every reader of its old content). */
int aqs_conv_push(const void *in, int64_t ld, int dtype, void *ring, const int32_t *slots, const int32_t *pos, int64_t B,
                  int64_t S, int64_t C, int64_t taps, void *stream);

/* ---- gated delta rule; state [slots, H, E, D] fp32 */
/* Convolution + SiLU of q | k | v (G, G heads of D, H of E), unit q (times D^-1/2) and k; decay =
 * exp(-exp(a_log) softplus(raw + dt_bias)) [M, H, D]; beta = sigmoid(beta_raw) [M, H]. */
int aqs_delta_prep(const void *qkv, int64_t ld, const void *raw, int64_t ld_raw, const void *beta_raw, int64_t ld_beta, int dtype,
                   const float *w, const void *ring, const int32_t *slots, const int32_t *pos, const float *a_log,
                   const float *dt_bias, float *q, float *k, float *v, float *decay, float *beta, int64_t B, int64_t S, int64_t H,
                   int64_t G, int64_t D, int64_t E, int64_t taps, void *stream);
int aqs_delta_scan(const float *q, const float *k, const float *v, const float *decay, const float *beta, float *state,
                   const int32_t *slots, const int32_t *pos, float *out, int64_t B, int64_t S, int64_t H, int64_t G, int64_t D,
                   int64_t E, void *stream);
/* One token per sequence, from the fused projection's row to the gated, normed head outputs.  a2 [H*D, rank_a] and
 * g2 [H*E, rank_g] are the second factors of the decay and of the output gate. */
int aqs_delta_step(const void *proj, int64_t ld, int64_t o_qkv, int64_t o_beta, int64_t o_a1, int64_t o_g1, int dtype,
                   const float *conv_w, void *ring, const int32_t *slots, const int32_t *pos, const void *a2, int64_t rank_a,
                   const void *g2, int64_t rank_g, const float *a_log, const float *dt_bias, const float *norm, float eps,
                   float out_scale, float *state, void *out, int64_t ldo, int64_t B, int64_t H, int64_t G, int64_t D, int64_t E,
                   int64_t taps, void *stream);

/* ---- state-space recurrence; state [slots, H, P, N] fp32; xbc [M, H*P | G*N | G*N] after convolution and SiLU */
int aqs_ssd_scan(const float *xbc, const void *dt_raw, int64_t ld_dt, int dtype, const float *dt_bias, const float *a_log,
                 const float *skip, float *state, const int32_t *slots, const int32_t *pos, float *out, int64_t B, int64_t S,
                 int64_t H, int64_t G, int64_t N, int64_t P, void *stream);
int aqs_ssd_step(const void *proj, int64_t ld, int64_t o_xbc, int64_t o_dt, int dtype, const float *conv_w, const float *conv_b,
                 void *ring, const int32_t *slots, const int32_t *pos, const float *dt_bias, const float *a_log,
                 const float *skip, float *state, float *y, int64_t B, int64_t H, int64_t G, int64_t N, int64_t P, int64_t taps,
                 void *stream);

/* ---- both recurrences over long prompts, in chunks of 64 tokens, convolution included (call aqs_conv_push after).
 * Sizes: aqs_chunked_ok(D or N, taps).  ws: scratch of at least the *_ws functions' number of floats. */
int aqs_chunked_ok(int64_t rows, int64_t taps);
int64_t aqs_delta_chunked_ws(int64_t B, int64_t S, int64_t H, int64_t D, int64_t E);
int64_t aqs_ssd_chunked_ws(int64_t B, int64_t S, int64_t H, int64_t G, int64_t N);
/* aqs_delta_prep and aqs_delta_scan */
int aqs_delta_chunked(const void *qkv, int64_t ld, const void *raw, int64_t ld_raw, const void *beta_raw, int64_t ld_beta,
                      int dtype, const float *w, const void *ring, const int32_t *slots, const int32_t *pos, const float *a_log,
                      const float *dt_bias, float *ws, int64_t ws_floats, float *state, float *out, int64_t B, int64_t S, int64_t H,
                      int64_t G, int64_t D, int64_t E, int64_t taps, void *stream);
/* aqs_conv_silu and aqs_ssd_scan; xbc: the raw projection columns x | B | C */
int aqs_ssd_chunked(const void *xbc, int64_t ld, const void *dt_raw, int64_t ld_dt, int dtype, const float *conv_w,
                    const float *conv_b, const void *ring, const int32_t *slots, const int32_t *pos, const float *dt_bias,
                    const float *a_log, const float *skip, float *ws, int64_t ws_floats, float *state, float *out, int64_t B,
                    int64_t S, int64_t H, int64_t G, int64_t N, int64_t P, int64_t taps, void *stream);

/* ---- sliding-window attention on pages: kc [n_pages, page, G, D], vc [n_pages, page, G, E], table [B, P] */
/* RMS norm (plain weight) and interleaved rotation of the first `rot` dimensions of q and k; q -> q_out [M, H, D],
 * k and v into their page slots.  cs [max_pos, rot/2, 2]: cos and sin by position. */
int aqs_attn_prep(const void *proj, int64_t ld, int64_t o_q, int64_t o_k, int64_t o_v, int dtype, const float *q_norm,
                  const float *k_norm, float eps, const float *cs, int64_t max_pos, int64_t rot, const int32_t *pos,
                  const int64_t *table, int64_t P, int64_t page, int64_t n_pages, void *q_out, void *kc, void *vc, int64_t B,
                  int64_t S, int64_t H, int64_t G, int64_t D, int64_t E, void *stream);
int aqs_attn_window_ok(int dtype, int64_t D, int64_t E, int64_t page);
/* The S new tokens (already in the pages) over the last `window` positions each; out [M, H, E] times sigmoid(gate [M, H])
 * (NULL: none) times out_scale.  simple != 0: the kernel for any sizes even where the matrix-core kernel would serve. */
int aqs_attn_window(const void *q, const void *kc, const void *vc, int dtype, float scale, int64_t window, const void *gate,
                    int64_t ld_gate, float out_scale, const int32_t *pos, const int64_t *table, int64_t P, int64_t page,
                    int64_t n_pages, void *out, int64_t ldo, int64_t B, int64_t S, int64_t H, int64_t G, int64_t D, int64_t E,
                    int simple, void *stream);
int aqs_attn_decode_ok(int64_t D, int64_t E, int64_t page);
int64_t aqs_attn_decode_slices(int64_t window, int64_t capacity);
/* One token per sequence: what aqs_attn_prep and aqs_attn_window do, from the projection's row.  o_gate < 0: no gate.
 * part: scratch of B * H * slices * (E + 4) floats, slices = aqs_attn_decode_slices(window, P * page). */
int aqs_attn_decode(const void *proj, int64_t ld, int64_t o_q, int64_t o_k, int64_t o_v, int64_t o_gate, int dtype,
                    const float *q_norm, const float *k_norm, float eps, const float *cs, int64_t max_pos, int64_t rot, float scale,
                    int64_t window, float out_scale, const int32_t *pos, const int64_t *table, int64_t P, int64_t page,
                    int64_t n_pages, void *kc, void *vc, float *part, int64_t slices, void *out, int64_t ldo, int64_t B, int64_t H,
                    int64_t G, int64_t D, int64_t E, void *stream);

#ifdef __cplusplus
}
#endif
#endif
