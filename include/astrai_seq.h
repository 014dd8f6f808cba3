/*
 * astrai_seq -- C ABI of the kernels for decoders that mix linear recurrences with
 * sliding-window or latent attention and routed experts (libastrai_seq.so, gfx950).
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
/* A branch's output t = y + sum over j < top of routed[slots[m, j]] (y may be NULL, top 0), normed with weight `post` if that is
 * given; x += mult * t; out = x / sqrt(mean(x^2) + eps) * (w0 + w) (out may be NULL when there is a branch). */
int aqs_add_rmsnorm(float *x, const void *y, int64_t ldy, int dtype, const void *routed, const int32_t *slots, int64_t top,
                    const float *post, float mult, const float *w, float w0, float eps, void *out, int64_t M, int64_t K,
                    void *stream);
/* gu [M, 2F] = gate | up;  g = min(gate, limit), u = clamp(up, -limit, limit);  out = g sigmoid(1.702 g) (u + 1). */
int aqs_clamped_glu(const void *gu, int64_t ld, int dtype, float limit, void *out, int64_t M, int64_t F, void *stream);
/* gu [M, 2F] = gate | up;  out = silu(gate) * up. */
int aqs_silu_glu(const void *gu, int64_t ld, int dtype, void *out, int64_t M, int64_t F, void *stream);
/* out = y / sqrt(mean(y^2) + eps) * w * sigmoid(z), y [M, K] fp32. */
int aqs_norm_gate(const float *y, const void *z, int64_t ldz, int dtype, const float *w, float eps, void *out, int64_t ldo,
                  int64_t M, int64_t K, void *stream);
/* out = RMS over each of `groups` equal parts of y * silu(z), times w [K]. */
int aqs_gated_group_norm(const float *y, const void *z, int64_t ldz, int dtype, const float *w, float eps, void *out,
                         int64_t ldo, int64_t M, int64_t K, int64_t groups, void *stream);
/* Per head of o [M, H, E]: RMS over E, times w [E], times sigmoid(gate [M, H*E]), times scale. */
int aqs_head_norm_gate(const float *o, const void *gate, int64_t ldg, int dtype, const float *w, float eps, float scale,
                       void *out, int64_t ldo, int64_t M, int64_t H, int64_t E, void *stream);

/* ---- matrix-vector products of a decode step (w [N, K] of dtype)
 * in_kind  0: x of dtype [M, ldx]   1: RMSNorm of xf [M, K] with gain0 + gain
 *          2: gated group norm of xf [M, K] with z = x (stride ldx), gain [K], groups
 *          3: as 1, of x_out = xf + mult * (yf normed with weight post); x_out is written and must not be xf
 *          4: RMSNorm of x of dtype [M, ldx] with gain   5: RMSNorm of xf with gain, times sigmoid(x) (stride ldx)
 * out_kind 0: out of dtype (+ bias) 1: fp32 into res   2: res += mult * result
 *          3: clamped GLU of w's first N/2 rows (gate) and last N/2 rows (up), out [M, N/2]
 *          4: w's first `routers` rows as fp32 into res [M, routers]; silu(gate) * up of the other rows into out; the
 *             normed rows into h_out [M, K] of dtype
 * Pairs served: 0-0, 0-1, 0-2, 1-0, 1-1, 1-3, 2-2, 3-0, 3-1, 3-4, 4-0, 5-1; sizes: aqs_gemv_ok. */
int aqs_gemv_ok(int dtype, int64_t M, int64_t N, int64_t K);
int aqs_gemv(int in_kind, int out_kind, int dtype, const void *x, int64_t ldx, const float *xf, const float *yf, const float *post,
             float *x_out, const float *gain, float gain0, float eps, int64_t groups, const void *w, const float *bias, float mult,
             float limit, int64_t routers, float *res, void *out, int64_t ldo, void *h_out, int64_t M, int64_t N, int64_t K,
             void *stream);

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

/* ---- state-space recurrence; state [slots, H, P, N] fp32; xbc [M, H*P | G*N | G*N] after convolution and SiLU.
 * decay [H] (not NULL): constant decays, step size 1, and dt_raw, dt_bias and a_log are not read; skip may be NULL (0). */
int aqs_ssd_scan(const float *xbc, const void *dt_raw, int64_t ld_dt, int dtype, const float *dt_bias, const float *a_log,
                 const float *skip, const float *decay, float *state, const int32_t *slots, const int32_t *pos, float *out,
                 int64_t B, int64_t S, int64_t H, int64_t G, int64_t N, int64_t P, void *stream);
int aqs_ssd_step(const void *proj, int64_t ld, int64_t o_xbc, int64_t o_dt, int dtype, const float *conv_w, const float *conv_b,
                 void *ring, const int32_t *slots, const int32_t *pos, const float *dt_bias, const float *a_log,
                 const float *skip, const float *decay, float *state, float *y, int64_t B, int64_t H, int64_t G, int64_t N,
                 int64_t P, int64_t taps, void *stream);

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
                    const float *a_log, const float *skip, const float *decay, float *ws, int64_t ws_floats, float *state,
                    float *out, int64_t B, int64_t S, int64_t H, int64_t G, int64_t N, int64_t P, int64_t taps, void *stream);

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

/* ---- latent attention; kc [n_pages, page, R + rot]: a position's normed latent and its rotated key part.
 * Rotation: elements i and i + rd / 2 of the first rd of `rot`; cs [max_pos, rd / 2, 2]. */
/* Norms of the new tokens' query latents (columns o_q .. + QR) -> cq [M, QR], their cache rows (columns o_kv .. + R + rot) into the
 * pages.  packed (may be NULL) [B, rows, R + rot]: the positions that the new tokens' windows reach, in order, from the block
 * of 64 on in which the first one's window begins; zero past the last token. */
int aqs_latent_prep(const void *proj, int64_t ld, int64_t o_q, int64_t o_kv, int dtype, const float *q_norm, const float *kv_norm,
                    float eps, const float *cs, int64_t max_pos, const int32_t *pos, const int64_t *table, int64_t P, int64_t page,
                    int64_t n_pages, int64_t window, void *cq, void *kc, void *packed, int64_t rows, int64_t B, int64_t S,
                    int64_t QR, int64_t R, int64_t rot, int64_t rd, void *stream);
/* The rotated part of every head of q [M, H, dim + rot], in place. */
int aqs_latent_rotate(void *q, int dtype, const float *cs, int64_t max_pos, const int32_t *pos, int64_t B, int64_t S, int64_t H,
                      int64_t dim, int64_t rot, int64_t rd, void *stream);
/* The new tokens' windows over packed rows: kv [B * rows, ld_kv] = keys' unrotated parts head by head | values head by head,
 * rotated parts in packed's columns o_rot .. + rot; out [M, H, E] times sigmoid(gate [M, H * E]). */
int aqs_latent_window(const void *q, const void *kv, int64_t ld_kv, const void *packed, int64_t ld_packed, int64_t o_rot, int dtype,
                      float scale, int64_t window, const void *gate, int64_t ld_gate, const int32_t *pos, int64_t rows, void *out,
                      int64_t ldo, int64_t B, int64_t S, int64_t H, int64_t dim, int64_t rot, int64_t E, int simple, void *stream);
int aqs_latent_decode_ok(int64_t B, int64_t dim, int64_t rot, int64_t R, int64_t E, int64_t page);
int64_t aqs_latent_decode_slices(int64_t window, int64_t capacity);
/* One token per sequence, from the projection's row and q [B, H, dim + rot] before rotation: page row, W_uk [H * dim, R] on the
 * query, attention, W_uv [H * E, R], gate (columns o_gate .. + H * E).  Scratch: qa of B * H * (R + rot) elements, part of
 * B * H * slices * (R + 4) floats, slices = aqs_latent_decode_slices(window, P * page). */
int aqs_latent_decode(const void *proj, int64_t ld, int64_t o_kv, int64_t o_gate, const void *q, const void *uk, const void *uv, int dtype,
                      const float *kv_norm, float eps, const float *cs, int64_t max_pos, float scale, int64_t window,
                      const int32_t *pos, const int64_t *table, int64_t P, int64_t page, int64_t n_pages, void *kc, void *qa,
                      float *part, int64_t slices, void *out, int64_t ldo, int64_t B, int64_t H, int64_t dim, int64_t rot, int64_t rd,
                      int64_t R, int64_t E, void *stream);

/* ---- routed experts (scores sigmoid(<router, h>), not renormalised; the score scales the expert's input) */
/* The `top` best of Ex experts of every row of h: ids and scores [M, top]. */
int aqs_moe_route(const void *h, int64_t ldh, int dtype, const void *w, int32_t *ids, float *scores, int64_t M, int64_t K, int64_t Ex,
                  int64_t top, void *stream);
/* Slots per tile for A choices among Ex experts of width K and inner size F; rows of `tiles` to make room for. */
int64_t aqs_moe_tile(int dtype, int64_t A, int64_t Ex, int64_t K, int64_t F);
int64_t aqs_moe_tiles(int64_t A, int64_t Ex, int64_t tile);
/* A choices (ids) by expert: rows[slot] = choice, slots[choice] = slot; tiles [n_tiles, 4]: how many there are, then expert, first
 * slot and number of slots of each. */
int aqs_moe_sort(const int32_t *ids, int64_t A, int64_t Ex, int64_t tile, int32_t *rows, int32_t *slots, int32_t *tiles,
                 int64_t n_tiles, void *stream);
/* glu != 0: x by token [., ldx], w [Ex, N = 2F, K] = gate | up, out [A, F] = silu(s gate) * (s up); 0: x by slot [A, ldx],
 * w [Ex, N, K], out [A, N]. */
int aqs_moe_product(int glu, const void *x, int64_t ldx, int dtype, const void *w, const int32_t *tiles, int64_t n_tiles, int64_t tile,
                    const int32_t *rows, const float *scores, int64_t A, int64_t top, void *out, int64_t N, int64_t K, void *stream);
/* A step of up to 8 tokens from the router's logits z [M, Ex]: act [M * top, F] of the chosen experts (w [Ex, 2F, K]), then
 * y [M, N] fp32 = sum of their down projections (w [Ex, N, F]) and of the shared expert's (sact [M, Fs], sw [N, Fs]; Fs 0: none). */
int aqs_moe_step_ok(int64_t M, int64_t N, int64_t F, int64_t Fs, int64_t Ex, int64_t top);
int aqs_moe_step_up(const void *h, const float *z, int dtype, const void *w, void *act, int64_t M, int64_t K, int64_t F, int64_t Ex,
                    int64_t top, void *stream);
int aqs_moe_step_down(const float *z, const void *act, int dtype, const void *w, const void *sact, const void *sw, float *y, int64_t M,
                      int64_t N, int64_t F, int64_t Fs, int64_t Ex, int64_t top, void *stream);

#ifdef __cplusplus
}
#endif
#endif
