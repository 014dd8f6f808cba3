// Linear recurrences with a matrix state per head, over the new tokens of every sequence:
//
//   gated delta rule   S <- g S (one decay per key channel), u = beta (v - S^T k), S <- S + k u^T, o = S^T q
//   state space (SSD)  S <- a S (one decay per head),        u = dt x,             S <- S + B u^T, y = S^T C + D x
//                      (with constant decays, dt = 1 and D = 0 it is linear attention: x = v, B = k, C = q)
//
// Both are "decay the rows, add an outer product, read out", so they share the scan kernel: rows of the state
// belong to k (or B), columns to v (or x).  The state is fp32 and is stored column by column, [slot, head, column,
// row]: the wavefront layout below then loads and stores it in whole contiguous lines.
//
//   A column is spread over a row of 16 lanes, RP state rows in each; a wavefront holds 4 columns and keeps them
//   in registers from the first token to the last.  The dot products over the rows end in four DPP adds.  Columns
//   never meet, so a head's columns go to different workgroups.
//
// In front of the scan: the causal per-channel convolutions with SiLU, unit norms, decays.  A sequence's last
// `taps - 1` convolution inputs live in a ring [slot, taps, channel], the input of position p in place p % taps: a
// single-token step writes only the place of its own position, which no reader of that step looks at.  A sequence
// that starts (position 0) reads neither ring nor state, so slots need no clearing.
#include "seq_common.h"

namespace sq {

// ---------------------------------------------------------------------------------------------- convolution
struct ConvSrc {
  const float* w;      // [C, taps], last column: the current token's
  const float* bias;   // [C] or null
  int C, taps;
};

// input of channel c at absolute position a (< 0: before the start)
template <typename T>
__device__ __forceinline__ float conv_in(const T* in, int64_t ld, int64_t tok0, int pos, const T* ring, int taps, int C, int c, int a) {
  if (a < 0) return 0.0f;
  if (a >= pos) return to_f32(in[(tok0 + (a - pos)) * ld + c]);
  return to_f32(ring[(int64_t)(a % taps) * C + c]);
}
template <typename T>
__device__ __forceinline__ float conv_at(const ConvSrc& s, const T* in, int64_t ld, int64_t tok0, int pos, const T* ring, int c, int p) {
  float acc = s.bias ? s.bias[c] : 0.0f;
  for (int j = 0; j < s.taps; ++j)
    acc = fmaf(s.w[c * s.taps + j], conv_in(in, ld, tok0, pos, ring, s.taps, s.C, c, p - (s.taps - 1) + j), acc);
  return acc;
}

// The same for the single token of a step at position pos (row: its inputs, channel c).  Up to four taps are requested at
// once at addresses that are always valid: a load under a condition would be waited for where the condition ends.
template <typename T>
__device__ __forceinline__ float conv_step(const ConvSrc& s, const T* row, int pos, const T* ring, int c) {
  if (s.taps > 4) return conv_at(s, row, 0, 0, pos, ring, c, pos);
  T x[4];
  float w[4];
#pragma unroll
  for (int back = 0; back < 4; ++back) {
    const bool on = back < s.taps && back <= pos;
    const int slot = on && back ? (pos - back) % s.taps : 0;
    const T* src = back ? ring + (int64_t)slot * s.C + c : row + c;
    x[back] = *src;
    const float v = s.w[c * s.taps + (back < s.taps ? s.taps - 1 - back : 0)];
    w[back] = on ? v : 0.0f;
  }
  float acc = s.bias ? s.bias[c] : 0.0f;
#pragma unroll
  for (int back = 3; back >= 0; --back) acc = w[back] != 0.0f ? fmaf(w[back], to_f32(x[back]), acc) : acc;
  return acc;
}

// out[m, c] = silu(conv) in fp32
template <typename T>
__global__ __launch_bounds__(256) void conv_silu_kernel(const T* in, int64_t ld, ConvSrc s, const T* ring, const int* slots,
                                                        const int* pos, float* out, int S) {
  const int nblk = (s.C + 255) / 256;
  const int c = (blockIdx.x % nblk) * 256 + threadIdx.x;
  if (c >= s.C) return;
  const int64_t m = blockIdx.x / nblk;
  const int b = (int)(m / S), t = (int)(m % S), p0 = pos[b];
  const float v = conv_at(s, in, ld, (int64_t)b * S, p0, ring + (int64_t)slots[b] * s.taps * s.C, c, p0 + t);
  out[m * s.C + c] = silu(v);
}

// the inputs of the last taps - 1 new tokens go into the ring
template <typename T>
__global__ __launch_bounds__(256) void conv_push_kernel(const T* in, int64_t ld, int C, int taps, T* ring, const int* slots,
                                                        const int* pos, int S) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= C) return;
  const int b = blockIdx.y, p0 = pos[b];
  T* r = ring + (int64_t)slots[b] * taps * C;
  const int n = S < taps - 1 ? S : taps - 1;
  for (int t = S - n; t < S; ++t) r[(int64_t)((p0 + t) % taps) * C + c] = in[((int64_t)b * S + t) * ld + c];
}

// ---------------------------------------------------------------------------------------------- delta: inputs
struct DeltaPrepArgs {
  ConvSrc s;             // channels q | k | v
  const int* slots;
  const int* pos;
  const float* a_log;    // [H]
  const float* dt_bias;  // [H * D]
  float* q;              // [M, G, D] unit vectors times D^-1/2
  float* k;              // [M, G, D] unit vectors
  float* v;              // [M, H, E]
  float* decay;          // [M, H, D], in (0, 1]
  float* beta;           // [M, H]
  int64_t M, ld, ld_raw, ld_beta;
  int S, H, G, D, E;
};
constexpr int PREP_MAX = 8;  // values per lane: head vectors of up to 512

// one wavefront per head vector of a token: G queries, G keys, H values, H decays (with beta)
template <typename T>
__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrepArgs p, const T* qkv, const T* raw, const T* b_raw, const T* ring) {
  const int items = 2 * p.G + 2 * p.H;
  const int64_t it = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (it >= p.M * items) return;
  const int64_t m = it / items;
  const int item = (int)(it % items), lane = threadIdx.x & 63;
  if (item >= 2 * p.G + p.H) {
    const int h = item - 2 * p.G - p.H;
    const float a = expf(p.a_log[h]);
    for (int d = lane; d < p.D; d += 64) {
      const int i = h * p.D + d;
      p.decay[m * p.H * p.D + i] = expf(-a * softplus(to_f32(raw[m * p.ld_raw + i]) + p.dt_bias[i]));
    }
    if (lane == 0) p.beta[m * p.H + h] = sigmoid(to_f32(b_raw[m * p.ld_beta + h]));
    return;
  }
  const bool is_v = item >= 2 * p.G;
  const int n = is_v ? p.E : p.D;
  const int c0 = is_v ? 2 * p.G * p.D + (item - 2 * p.G) * p.E : item * p.D;
  const int b = (int)(m / p.S), t = (int)(m % p.S), p0 = p.pos[b];
  const T* r = ring + (int64_t)p.slots[b] * p.s.taps * p.s.C;
  float x[PREP_MAX], ss = 0.0f;
#pragma unroll
  for (int i = 0; i < PREP_MAX; ++i) {
    const int d = i * 64 + lane;
    x[i] = d < n ? silu(conv_at(p.s, qkv, p.ld, (int64_t)b * p.S, p0, r, c0 + d, p0 + t)) : 0.0f;
    ss += x[i] * x[i];
  }
  float scale = 1.0f;
  if (!is_v) {
    scale = 1.0f / sqrtf(wave_sum(ss) + 1e-6f);
    if (item < p.G) scale /= sqrtf((float)p.D);
  }
  float* dst = is_v ? p.v + m * p.H * p.E + (item - 2 * p.G) * p.E
                    : (item < p.G ? p.q + (m * p.G + item) * p.D : p.k + (m * p.G + item - p.G) * p.D);
#pragma unroll
  for (int i = 0; i < PREP_MAX; ++i) {
    const int d = i * 64 + lane;
    if (d < n) dst[d] = x[i] * scale;
  }
}

// ---------------------------------------------------------------------------------------------- the scan
struct ScanArgs {
  const float* k;  // element (m, group, row) at k + m * ld_k + group * R + row; likewise q
  const float* q;
  const float* v;  // element (m, head, column) at v + m * ld_v + head * E + column
  const float* decay;    // delta: [M, H, R]; ssd: [H] if the decays are constants (step size 1), else null
  const float* beta;     // delta: [M, H]
  const float* dt_bias;  // ssd: [H]
  const float* a_log;    // ssd: [H]
  const float* skip;     // ssd: [H], the D of y = S^T C + D x
  float* state;          // [slots, H, E, R]
  float* out;            // [M, H, E]
  const int* slots;
  const int* pos;
  int64_t ld_k, ld_q, ld_v, ld_dt;
  int S, H, G, R, E;
};

constexpr int SCAN_TC = 16;    // tokens staged at a time
constexpr int SCAN_COLS = 16;  // columns per workgroup

template <int RP>
__device__ __forceinline__ float dot_rows(const float (&a)[RP], const float (&b)[RP]) {
  float s0 = a[0] * b[0], s1 = a[1] * b[1];
#pragma unroll
  for (int i = 2; i < RP; i += 2) {
    s0 = fmaf(a[i], b[i], s0);
    s1 = fmaf(a[i + 1], b[i + 1], s1);
  }
  return s0 + s1;
}
// RP state rows of one column from row r0 on; rows past R are zero
template <int RP>
__device__ __forceinline__ void load_rows(const float* col, int r0, int R, bool ok, float (&s)[RP]) {
  if (ok && R % RP == 0 && r0 < R) {
    load_vec<RP>(col + r0, s);
    return;
  }
#pragma unroll
  for (int i = 0; i < RP; ++i) s[i] = (ok && r0 + i < R) ? col[r0 + i] : 0.0f;
}
template <int RP>
__device__ __forceinline__ void store_rows(float* col, int r0, int R, const float (&s)[RP]) {
  if (R % RP == 0 && r0 < R) {
    if constexpr (RP % 4 == 0) {
#pragma unroll
      for (int i = 0; i < RP / 4; ++i)
        reinterpret_cast<float4*>(col + r0)[i] = make_float4(s[4 * i], s[4 * i + 1], s[4 * i + 2], s[4 * i + 3]);
    } else {
      *reinterpret_cast<float2*>(col + r0) = make_float2(s[0], s[1]);
    }
    return;
  }
#pragma unroll
  for (int i = 0; i < RP; ++i)
    if (r0 + i < R) col[r0 + i] = s[i];
}

template <bool DELTA, int RP, typename T>
__global__ __launch_bounds__(256) void scan_kernel(ScanArgs p, const T* dt_raw) {
  constexpr int DP = 16 * RP, TC = SCAN_TC, NA = DELTA ? 3 : 2;
  constexpr int F4 = TC * DP / 4;                 // float4 per staged array
  constexpr int PER = (F4 + 255) / 256;           // of them per thread
  __shared__ __align__(16) float rows_s[2][NA][TC * DP];
  __shared__ __align__(16) float v_s[2][TC][SCAN_COLS];
  __shared__ __align__(16) float2 c_s[2][TC];     // delta: (beta, -); ssd: (decay, dt)
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int tiles = (p.E + SCAN_COLS - 1) / SCAN_COLS;
  const int tile = blockIdx.x % tiles, h = (blockIdx.x / tiles) % p.H, b = blockIdx.x / (tiles * p.H);
  const int j = h / (p.H / p.G);
  const int r = lane & 15, r0 = r * RP, cl = wave * 4 + (lane >> 4), e = tile * SCAN_COLS + cl;
  const int64_t m0 = (int64_t)b * p.S;
  const int R = p.R;
  float* col = p.state + (((int64_t)p.slots[b] * p.H + h) * p.E + (e < p.E ? e : 0)) * R;
  float s[RP];
  load_rows<RP>(col, r0, R, e < p.E && p.pos[b] > 0, s);
  float skip = 0.0f, neg_a = 0.0f, dtb = 0.0f;
  const bool constant = !DELTA && p.decay;
  if constexpr (!DELTA) {
    skip = p.skip ? p.skip[h] : 0.0f;
    if (!constant) neg_a = -expf(p.a_log[h]), dtb = p.dt_bias[h];
  }
  const float* src[3] = {p.k + m0 * p.ld_k + (int64_t)j * R, p.q + m0 * p.ld_q + (int64_t)j * R,
                         DELTA ? p.decay + (m0 * p.H + h) * R : nullptr};
  const int64_t ld[3] = {p.ld_k, p.ld_q, (int64_t)p.H * R};
  const float* vsrc = p.v + m0 * p.ld_v + (int64_t)h * p.E + tile * SCAN_COLS;
  const bool vec = R % 4 == 0 && p.ld_k % 4 == 0 && p.ld_q % 4 == 0 && (((uintptr_t)p.k | (uintptr_t)p.q) & 15) == 0;

  float4 reg[NA][PER];
  float vreg = 0.0f;
  float2 creg = make_float2(0.0f, 0.0f);
  auto fetch = [&](int t0) __attribute__((always_inline)) {
#pragma unroll
    for (int a = 0; a < NA; ++a)
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const int idx = i * 256 + tid, t = idx / (DP / 4), d = (idx % (DP / 4)) * 4;
        float4 v = make_float4(0, 0, 0, 0);
        if (idx < F4 && t0 + t < p.S && d < R) {
          const float* q = src[a] + (int64_t)(t0 + t) * ld[a] + d;
          if (vec) {
            v = *reinterpret_cast<const float4*>(q);
          } else {
            v.x = q[0];
            if (d + 1 < R) v.y = q[1];
            if (d + 2 < R) v.z = q[2];
            if (d + 3 < R) v.w = q[3];
          }
        }
        reg[a][i] = v;
      }
    const int t = tid / SCAN_COLS, c = tid % SCAN_COLS;
    vreg = (t0 + t < p.S && tile * SCAN_COLS + c < p.E) ? vsrc[(int64_t)(t0 + t) * p.ld_v + c] : 0.0f;
    if (tid < TC && t0 + tid < p.S) {
      if constexpr (DELTA) {
        creg.x = p.beta[(m0 + t0 + tid) * p.H + h];
      } else if (constant) {
        creg = make_float2(p.decay[h], 1.0f);
      } else {
        const float dt = softplus(to_f32(dt_raw[(m0 + t0 + tid) * p.ld_dt + h]) + dtb);
        creg = make_float2(expf(neg_a * dt), dt);
      }
    }
  };
  auto stage = [&](int buf) __attribute__((always_inline)) {
#pragma unroll
    for (int a = 0; a < NA; ++a)
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const int idx = i * 256 + tid;
        if (idx < F4) reinterpret_cast<float4*>(rows_s[buf][a])[idx] = reg[a][i];
      }
    v_s[buf][tid / SCAN_COLS][tid % SCAN_COLS] = vreg;
    if (tid < TC) c_s[buf][tid] = creg;
  };
  auto tokens = [&](int buf, auto n_tag, int t0) __attribute__((always_inline)) {
    const int n = n_tag;  // an integral constant for a whole chunk
    float kept = 0.0f;
    float kn[RP], qn[RP], gn[RP], vn;
    float2 cn;
    auto read = [&](int t) __attribute__((always_inline)) {
      load_vec<RP>(&rows_s[buf][0][t * DP + r0], kn);
      load_vec<RP>(&rows_s[buf][1][t * DP + r0], qn);
      if constexpr (DELTA) load_vec<RP>(&rows_s[buf][NA - 1][t * DP + r0], gn);
      vn = v_s[buf][t][cl];
      cn = c_s[buf][t];
    };
    read(0);
    for (int t = 0; t < n; ++t) {
      float k[RP], q[RP], g[RP];
      const float v = vn;
      const float2 c = cn;
#pragma unroll
      for (int i = 0; i < RP; ++i) {
        k[i] = kn[i], q[i] = qn[i];
        if constexpr (DELTA) g[i] = gn[i];
      }
      read(t + 1 < TC ? t + 1 : t);
      float o;
      if constexpr (DELTA) {
#pragma unroll
        for (int i = 0; i < RP; ++i) s[i] *= g[i];
        const float u = c.x * (v - row16_sum(dot_rows<RP>(s, k)));
#pragma unroll
        for (int i = 0; i < RP; ++i) s[i] = fmaf(k[i], u, s[i]);
        o = row16_sum(dot_rows<RP>(s, q));
      } else {
        const float u = c.y * v;
#pragma unroll
        for (int i = 0; i < RP; ++i) s[i] = fmaf(k[i], u, c.x * s[i]);
        o = row16_sum(dot_rows<RP>(s, q)) + skip * v;
      }
      kept = r == t ? o : kept;  // lane r of the column's row keeps token r
    }
    if (r < n && e < p.E) p.out[((m0 + t0 + r) * p.H + h) * p.E + e] = kept;
  };
  fetch(0);
  int buf = 0;
  for (int t0 = 0; t0 < p.S; t0 += TC, buf ^= 1) {
    stage(buf);
    __syncthreads();
    if (t0 + TC < p.S) fetch(t0 + TC);
    const int n = p.S - t0 < TC ? p.S - t0 : TC;
    if (n == TC) tokens(buf, std::integral_constant<int, TC>{}, t0);
    else tokens(buf, n, t0);
  }
  if (e < p.E) store_rows<RP>(col, r0, R, s);
}

// ---------------------------------------------------------------------------------------------- single tokens
// A whole step of the delta mixer between its projections, one workgroup per (head, sequence): convolution of the
// head's q, k and v channels, unit norms, the two low-rank second factors (decay, output gate), the recurrence, the
// head's norm and gate.  proj is the row of the fused input projection; ring writes: q and k channels by the first
// head of each group.
struct DeltaStepArgs {
  ConvSrc s;
  const int* slots;
  const int* pos;
  const float* a_log;    // [H]
  const float* dt_bias;  // [H * D]
  const float* norm;     // [E]
  float* state;          // [slots, H, E, D]
  int64_t ld;            // of proj
  int64_t o_qkv, o_beta, o_a1, o_g1;  // columns of proj
  int64_t ldo;
  int H, G, D, E, rank_a, rank_g;  // ranks: multiples of 8 (zero padded)
  float eps, out_scale;
};

constexpr int STEP_WAVES = 8;
constexpr int STEP_MAX = 256;  // rows and columns of a head's state

// sum_k w[row, k] x[k] by four lanes (sub 0..3); every lane of the quad gets it.  n a multiple of 8.  Four pieces per
// lane are requested at once.
template <typename T>
__device__ __forceinline__ float quad_dot(const T* w, const T* x, int n, int sub) {
  float acc = 0.0f;
  for (int c0 = 0; c0 < n; c0 += 128) {
    Raw8<T> a[4], b[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = c0 + i * 32 + sub * 8;
      a[i].load(w + (c < n ? c : 0));
      b[i].load(x + (c < n ? c : 0));
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      float fa[8], fb[8], part = 0.0f;
      a[i].get(fa);
      b[i].get(fb);
#pragma unroll
      for (int e = 0; e < 8; ++e) part = fmaf(fa[e], fb[e], part);
      acc += c0 + i * 32 + sub * 8 < n ? part : 0.0f;
    }
  }
  SQ_DPP_ADD(acc, 0xB1);
  SQ_DPP_ADD(acc, 0x4E);
  return acc;
}

template <typename T, int RP, int NI>
__global__ __launch_bounds__(STEP_WAVES * 64) void delta_step_kernel(DeltaStepArgs p, const T* proj, T* ring, const T* a2,
                                                                     const T* g2, T* out) {
  constexpr int TH = STEP_WAVES * 64, CPI = STEP_WAVES * 4;  // columns per iteration
  __shared__ __align__(16) float q_s[STEP_MAX], k_s[STEP_MAX], g_s[STEP_MAX];
  __shared__ float v_s[STEP_MAX], o_s[STEP_MAX], gate_s[STEP_MAX], red[STEP_WAVES];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = blockIdx.x, b = blockIdx.y, per = p.H / p.G, j = h / per;
  const int slot = p.slots[b], pos = p.pos[b], D = p.D, E = p.E;
  const int r0 = (lane & 15) * RP, cl = wave * 4 + (lane >> 4);
  const T* row = proj + b * p.ld;
  float* st = p.state + ((int64_t)slot * p.H + h) * E * D;
  float s[NI][RP];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int e = i * CPI + cl;
    load_rows<RP>(st + (int64_t)e * D, r0, D, e < E && pos > 0, s[i]);
  }
  // rows past D take part in the dot products: zero in all three
  for (int d = tid; d < STEP_MAX; d += TH)
    if (d >= D) q_s[d] = k_s[d] = g_s[d] = 0.0f;
  T* rg = ring + (int64_t)slot * p.s.taps * p.s.C;
  const T* cin = row + p.o_qkv;
  for (int i = tid; i < 2 * D + E; i += TH) {
    const int which = i < D ? 0 : i < 2 * D ? 1 : 2;
    const int d = i - which * D;
    const int c = which == 2 ? 2 * p.G * D + h * E + d : (which * p.G + j) * D + d;
    const float x = silu(conv_step(p.s, cin, pos, rg, c));
    (which == 0 ? q_s : which == 1 ? k_s : v_s)[d] = x;
    if (which == 2 || h % per == 0) rg[(int64_t)(pos % p.s.taps) * p.s.C + c] = cin[c];
  }
  const float a = expf(p.a_log[h]);
  for (int d0 = 0; d0 < D; d0 += TH / 4) {
    const int d = d0 + tid / 4;
    const float raw = quad_dot<T>(a2 + (int64_t)(h * D + (d < D ? d : 0)) * p.rank_a, row + p.o_a1, p.rank_a, tid & 3);
    if (d < D && (tid & 3) == 0) g_s[d] = expf(-a * softplus(raw + p.dt_bias[h * D + d]));
  }
  for (int e0 = 0; e0 < E; e0 += TH / 4) {
    const int e = e0 + tid / 4;
    const float raw = quad_dot<T>(g2 + (int64_t)(h * E + (e < E ? e : 0)) * p.rank_g, row + p.o_g1, p.rank_g, tid & 3);
    if (e < E && (tid & 3) == 0) gate_s[e] = sigmoid(raw);
  }
  const float beta = sigmoid(to_f32(row[p.o_beta + h]));
  __syncthreads();
  if (wave < 2) {
    float* x = wave == 0 ? q_s : k_s;
    float ss = 0.0f;
    for (int d = lane; d < D; d += 64) ss += x[d] * x[d];
    ss = wave_sum(ss);
    float scale = 1.0f / sqrtf(ss + 1e-6f);
    if (wave == 0) scale /= sqrtf((float)D);
    for (int d = lane; d < D; d += 64) x[d] *= scale;
  }
  __syncthreads();
  float k[RP], q[RP], g[RP];
  load_vec<RP>(&k_s[r0], k);
  load_vec<RP>(&q_s[r0], q);
  load_vec<RP>(&g_s[r0], g);
  float ss = 0.0f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int e = i * CPI + cl;
    if (i * CPI >= E) break;
#pragma unroll
    for (int x = 0; x < RP; ++x) s[i][x] *= g[x];
    const float u = beta * ((e < E ? v_s[e] : 0.0f) - row16_sum(dot_rows<RP>(s[i], k)));
#pragma unroll
    for (int x = 0; x < RP; ++x) s[i][x] = fmaf(k[x], u, s[i][x]);
    const float o = row16_sum(dot_rows<RP>(s[i], q));
    if (e < E) {
      store_rows<RP>(st + (int64_t)e * D, r0, D, s[i]);
      if ((lane & 15) == 0) {
        o_s[e] = o;
        ss += o * o;
      }
    }
  }
  ss = block_sum<STEP_WAVES>(ss, red);
  const float rn = 1.0f / sqrtf(ss / (float)E + p.eps);
  for (int e = tid; e < E; e += TH) out[b * p.ldo + h * E + e] = from_f32<T>(o_s[e] * rn * p.norm[e] * gate_s[e] * p.out_scale);
}

// The same for the state-space mixer, up to the gated norm (which spans heads): convolution of the head's x channels
// and its group's B and C, step size, recurrence.  y fp32 [B, H * P].
struct SsdStepArgs {
  ConvSrc s;  // channels x | B | C
  const int* slots;
  const int* pos;
  const float* dt_bias;
  const float* a_log;
  const float* skip;     // or null
  const float* decay;    // [H] constant decays (step size 1), or null
  float* state;  // [slots, H, P, N]
  float* y;
  int64_t ld, o_xbc, o_dt;
  int H, G, N, P;
};

constexpr int SSD_STEP_COLS = 32;  // state columns per workgroup: a head's columns never meet

template <typename T, int RP, int NI>
__global__ __launch_bounds__(256) void ssd_step_kernel(SsdStepArgs p, const T* proj, T* ring) {
  constexpr int TH = 256, CPI = 16;
  __shared__ __align__(16) float b_s[STEP_MAX], c_s[STEP_MAX];
  __shared__ float x_s[NI * CPI];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int tiles = (p.P + NI * CPI - 1) / (NI * CPI), h = blockIdx.x / tiles, e0 = (blockIdx.x % tiles) * NI * CPI;
  const int b = blockIdx.y, per = p.H / p.G, j = h / per, cols = p.P - e0 < NI * CPI ? p.P - e0 : NI * CPI;
  const int slot = p.slots[b], pos = p.pos[b], N = p.N, P = p.P, inner = p.H * P;
  const int r0 = (lane & 15) * RP, cl = wave * 4 + (lane >> 4);
  const T* row = proj + b * p.ld;
  float* st = p.state + (((int64_t)slot * p.H + h) * P + e0) * N;
  float s[NI][RP];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int e = i * CPI + cl;
    load_rows<RP>(st + (int64_t)e * N, r0, N, e < cols && pos > 0, s[i]);
  }
  for (int d = tid; d < STEP_MAX; d += TH)
    if (d >= N) b_s[d] = c_s[d] = 0.0f;
  T* rg = ring + (int64_t)slot * p.s.taps * p.s.C;
  const T* cin = row + p.o_xbc;
  for (int i = tid; i < 2 * N + cols; i += TH) {
    const int which = i < N ? 0 : i < 2 * N ? 1 : 2;
    const int d = i - which * N;
    const int c = which == 2 ? h * P + e0 + d : inner + (which * p.G + j) * N + d;
    const float x = silu(conv_step(p.s, cin, pos, rg, c));
    (which == 0 ? b_s : which == 1 ? c_s : x_s)[d] = x;
    if (which == 2 || (h % per == 0 && e0 == 0)) rg[(int64_t)(pos % p.s.taps) * p.s.C + c] = cin[c];
  }
  const float dt = p.decay ? 1.0f : softplus(to_f32(row[p.o_dt + h]) + p.dt_bias[h]);
  const float a = p.decay ? p.decay[h] : expf(-expf(p.a_log[h]) * dt), skip = p.skip ? p.skip[h] : 0.0f;
  __syncthreads();
  float k[RP], q[RP];
  load_vec<RP>(&b_s[r0], k);
  load_vec<RP>(&c_s[r0], q);
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int e = i * CPI + cl;
    if (i * CPI >= cols) break;
    const float x = e < cols ? x_s[e] : 0.0f, u = dt * x;
#pragma unroll
    for (int w = 0; w < RP; ++w) s[i][w] = fmaf(k[w], u, a * s[i][w]);
    const float o = row16_sum(dot_rows<RP>(s[i], q)) + skip * x;
    if (e < cols) {
      store_rows<RP>(st + (int64_t)e * N, r0, N, s[i]);
      if ((lane & 15) == 0) p.y[(int64_t)b * inner + h * P + e0 + e] = o;
    }
  }
}

}  // namespace sq

using namespace sq;

// RP: state rows per lane for R rows
#define SQ_ROWS(R, CALL)                 \
  do {                                   \
    if ((R) <= 32) {                     \
      constexpr int RP = 2;              \
      CALL;                              \
    } else if ((R) <= 64) {              \
      constexpr int RP = 4;              \
      CALL;                              \
    } else if ((R) <= 128) {             \
      constexpr int RP = 8;              \
      CALL;                              \
    } else {                             \
      constexpr int RP = 16;             \
      CALL;                              \
    }                                    \
  } while (0)
// NI: iterations of CPI columns each
#define SQ_ITERS(n, CALL)                \
  do {                                   \
    if ((n) <= 1) {                      \
      constexpr int NI = 1;              \
      CALL;                              \
    } else if ((n) <= 2) {               \
      constexpr int NI = 2;              \
      CALL;                              \
    } else if ((n) <= 4) {               \
      constexpr int NI = 4;              \
      CALL;                              \
    } else if ((n) <= 8) {               \
      constexpr int NI = 8;              \
      CALL;                              \
    } else {                             \
      constexpr int NI = 16;             \
      CALL;                              \
    }                                    \
  } while (0)

extern "C" int aqs_conv_silu(const void* in, int64_t ld, int dtype, const float* w, const float* bias, const void* ring,
                             const int32_t* slots, const int32_t* pos, float* out, int64_t B, int64_t S, int64_t C, int64_t taps,
                             void* stream) {
  SQ_CHECK(B >= 0 && S >= 0 && C > 0 && taps > 0 && ld >= C, AQ_E_SHAPE);
  SQ_CHECK(B * S < ((int64_t)1 << 31) && C < (1 << 24) && taps <= 64, AQ_E_RANGE);
  if (B * S == 0) return AQ_OK;
  SQ_NEED(in && w && ring && slots && pos && out);
  const ConvSrc s{w, bias, (int)C, (int)taps};
  // gridDim.y is limited to 65535: longer batches go in pieces of whole sequences by the caller
  SQ_CHECK(B * S * ((C + 255) / 256) < (1 << 24), AQ_E_RANGE);  // a launch holds fewer than 2^32 threads
  const dim3 grid((unsigned)(B * S * ((C + 255) / 256)));
  SQ_DISPATCH(dtype, (conv_silu_kernel<T><<<grid, 256, 0, (hipStream_t)stream>>>((const T*)in, ld, s, (const T*)ring, slots, pos,
                                                                                 out, (int)S)));
  return launched();
}

extern "C" int aqs_conv_push(const void* in, int64_t ld, int dtype, void* ring, const int32_t* slots, const int32_t* pos,
                             int64_t B, int64_t S, int64_t C, int64_t taps, void* stream) {
  SQ_CHECK(B >= 0 && S >= 0 && C > 0 && taps > 0 && ld >= C, AQ_E_SHAPE);
  SQ_CHECK(B <= 65535 && S < ((int64_t)1 << 31) && C < (1 << 24) && taps <= 64, AQ_E_RANGE);
  if (B * S == 0 || taps == 1) return AQ_OK;
  SQ_NEED(in && ring && slots && pos);
  const dim3 grid((unsigned)((C + 255) / 256), (unsigned)B);
  SQ_DISPATCH(dtype, (conv_push_kernel<T><<<grid, 256, 0, (hipStream_t)stream>>>((const T*)in, ld, (int)C, (int)taps, (T*)ring,
                                                                                 slots, pos, (int)S)));
  return launched();
}

extern "C" int aqs_delta_prep(const void* qkv, int64_t ld, const void* raw, int64_t ld_raw, const void* beta_raw, int64_t ld_beta,
                              int dtype, const float* w, const void* ring, const int32_t* slots, const int32_t* pos,
                              const float* a_log, const float* dt_bias, float* q, float* k, float* v, float* decay, float* beta,
                              int64_t B, int64_t S, int64_t H, int64_t G, int64_t D, int64_t E, int64_t taps, void* stream) {
  SQ_CHECK(B >= 0 && S >= 0 && H > 0 && G > 0 && H % G == 0 && D > 0 && E > 0 && taps > 0, AQ_E_SHAPE);
  SQ_CHECK(D <= 64 * PREP_MAX && E <= 64 * PREP_MAX && taps <= 64, AQ_E_RANGE);
  SQ_CHECK(ld >= 2 * G * D + H * E && ld_raw >= H * D && ld_beta >= H, AQ_E_SHAPE);
  SQ_CHECK(B * S * (2 * G + 2 * H) < ((int64_t)1 << 26), AQ_E_RANGE);  // a launch holds fewer than 2^32 threads
  if (B * S == 0) return AQ_OK;
  SQ_NEED(qkv && raw && beta_raw && w && ring && slots && pos && a_log && dt_bias && q && k && v && decay && beta);
  DeltaPrepArgs a{};
  a.s = ConvSrc{w, nullptr, (int)(2 * G * D + H * E), (int)taps};
  a.slots = slots, a.pos = pos, a.a_log = a_log, a.dt_bias = dt_bias;
  a.q = q, a.k = k, a.v = v, a.decay = decay, a.beta = beta;
  a.M = B * S, a.ld = ld, a.ld_raw = ld_raw, a.ld_beta = ld_beta;
  a.S = (int)S, a.H = (int)H, a.G = (int)G, a.D = (int)D, a.E = (int)E;
  const unsigned grid = (unsigned)((a.M * (2 * G + 2 * H) + 3) / 4);
  SQ_DISPATCH(dtype, (delta_prep_kernel<T><<<grid, 256, 0, (hipStream_t)stream>>>(a, (const T*)qkv, (const T*)raw,
                                                                                  (const T*)beta_raw, (const T*)ring)));
  return launched();
}

extern "C" int aqs_delta_scan(const float* q, const float* k, const float* v, const float* decay, const float* beta, float* state,
                              const int32_t* slots, const int32_t* pos, float* out, int64_t B, int64_t S, int64_t H, int64_t G,
                              int64_t D, int64_t E, void* stream) {
  SQ_CHECK(B >= 0 && S >= 0 && H > 0 && G > 0 && H % G == 0 && D > 0 && E > 0, AQ_E_SHAPE);
  SQ_CHECK(D <= STEP_MAX && S < ((int64_t)1 << 31), AQ_E_RANGE);
  if (B * S == 0) return AQ_OK;
  SQ_NEED(q && k && v && decay && beta && state && slots && pos && out);
  ScanArgs a{};
  a.k = k, a.q = q, a.v = v, a.decay = decay, a.beta = beta, a.state = state, a.out = out, a.slots = slots, a.pos = pos;
  a.ld_k = a.ld_q = G * D, a.ld_v = H * E;
  a.S = (int)S, a.H = (int)H, a.G = (int)G, a.R = (int)D, a.E = (int)E;
  const int64_t grid = B * H * ((E + SCAN_COLS - 1) / SCAN_COLS);
  SQ_CHECK(grid < (1 << 24), AQ_E_RANGE);
  SQ_ROWS(D, (scan_kernel<true, RP, float><<<dim3((unsigned)grid), 256, 0, (hipStream_t)stream>>>(a, nullptr)));
  return launched();
}

extern "C" int aqs_ssd_scan(const float* xbc, const void* dt_raw, int64_t ld_dt, int dtype, const float* dt_bias, const float* a_log,
                            const float* skip, const float* decay, float* state, const int32_t* slots, const int32_t* pos, float* out,
                            int64_t B, int64_t S, int64_t H, int64_t G, int64_t N, int64_t P, void* stream) {
  SQ_CHECK(B >= 0 && S >= 0 && H > 0 && G > 0 && H % G == 0 && N > 0 && P > 0 && (decay || ld_dt >= H), AQ_E_SHAPE);
  SQ_CHECK(N <= STEP_MAX && S < ((int64_t)1 << 31), AQ_E_RANGE);
  if (B * S == 0) return AQ_OK;
  SQ_NEED(xbc && (decay || (dt_raw && dt_bias && a_log)) && state && slots && pos && out);
  ScanArgs a{};
  const int64_t C = H * P + 2 * G * N;
  a.v = xbc, a.k = xbc + H * P, a.q = xbc + H * P + G * N;
  a.dt_bias = dt_bias, a.a_log = a_log, a.skip = skip, a.decay = decay, a.state = state, a.out = out, a.slots = slots, a.pos = pos;
  a.ld_k = a.ld_q = a.ld_v = C, a.ld_dt = ld_dt;
  a.S = (int)S, a.H = (int)H, a.G = (int)G, a.R = (int)N, a.E = (int)P;
  const int64_t grid = B * H * ((P + SCAN_COLS - 1) / SCAN_COLS);
  SQ_CHECK(grid < (1 << 24), AQ_E_RANGE);
  SQ_DISPATCH(dtype, SQ_ROWS(N, (scan_kernel<false, RP, T><<<dim3((unsigned)grid), 256, 0, (hipStream_t)stream>>>(a, (const T*)dt_raw))));
  return launched();
}

extern "C" int aqs_delta_step(const void* proj, int64_t ld, int64_t o_qkv, int64_t o_beta, int64_t o_a1, int64_t o_g1, int dtype,
                              const float* conv_w, void* ring, const int32_t* slots, const int32_t* pos, const void* a2,
                              int64_t rank_a, const void* g2, int64_t rank_g, const float* a_log, const float* dt_bias,
                              const float* norm, float eps, float out_scale, float* state, void* out, int64_t ldo, int64_t B,
                              int64_t H, int64_t G, int64_t D, int64_t E, int64_t taps, void* stream) {
  SQ_CHECK(B >= 0 && H > 0 && G > 0 && H % G == 0 && D > 0 && E > 0 && taps > 0 && rank_a > 0 && rank_g > 0, AQ_E_SHAPE);
  SQ_CHECK(rank_a % 8 == 0 && rank_g % 8 == 0 && ld % 8 == 0 && o_a1 % 8 == 0 && o_g1 % 8 == 0, AQ_E_SHAPE);
  SQ_CHECK(D <= STEP_MAX && E <= STEP_MAX && taps <= 64 && B <= 65535, AQ_E_RANGE);
  SQ_CHECK(o_qkv >= 0 && o_beta >= 0 && o_a1 >= 0 && o_g1 >= 0 && o_qkv + 2 * G * D + H * E <= ld && o_beta + H <= ld &&
               o_a1 + rank_a <= ld && o_g1 + rank_g <= ld && ldo >= H * E, AQ_E_SHAPE);
  if (B == 0) return AQ_OK;
  SQ_NEED(proj && conv_w && ring && slots && pos && a2 && g2 && a_log && dt_bias && norm && state && out);
  SQ_CHECK(!bad_ptr16(proj) && !bad_ptr16(a2) && !bad_ptr16(g2) && !bad_ptr16(state), AQ_E_ALIGN);
  DeltaStepArgs a{};
  a.s = ConvSrc{conv_w, nullptr, (int)(2 * G * D + H * E), (int)taps};
  a.slots = slots, a.pos = pos, a.a_log = a_log, a.dt_bias = dt_bias, a.norm = norm, a.state = state;
  a.ld = ld, a.o_qkv = o_qkv, a.o_beta = o_beta, a.o_a1 = o_a1, a.o_g1 = o_g1, a.ldo = ldo;
  a.H = (int)H, a.G = (int)G, a.D = (int)D, a.E = (int)E, a.rank_a = (int)rank_a, a.rank_g = (int)rank_g;
  a.eps = eps, a.out_scale = out_scale;
  const dim3 grid((unsigned)H, (unsigned)B);
  const int64_t iters = (E + STEP_WAVES * 4 - 1) / (STEP_WAVES * 4);
  SQ_DISPATCH(dtype, SQ_ROWS(D, SQ_ITERS(iters, (delta_step_kernel<T, RP, (NI > 8 ? 8 : NI)><<<grid, STEP_WAVES * 64, 0, (hipStream_t)stream>>>(
                         a, (const T*)proj, (T*)ring, (const T*)a2, (const T*)g2, (T*)out)))));
  return launched();
}

extern "C" int aqs_ssd_step(const void* proj, int64_t ld, int64_t o_xbc, int64_t o_dt, int dtype, const float* conv_w,
                            const float* conv_b, void* ring, const int32_t* slots, const int32_t* pos, const float* dt_bias,
                            const float* a_log, const float* skip, const float* decay, float* state, float* y, int64_t B,
                            int64_t H, int64_t G, int64_t N, int64_t P, int64_t taps, void* stream) {
  SQ_CHECK(B >= 0 && H > 0 && G > 0 && H % G == 0 && N > 0 && P > 0 && taps > 0, AQ_E_SHAPE);
  SQ_CHECK(N <= STEP_MAX && P <= STEP_MAX && taps <= 64 && B <= 65535, AQ_E_RANGE);
  SQ_CHECK(o_xbc >= 0 && o_xbc + H * P + 2 * G * N <= ld && (decay || (o_dt >= 0 && o_dt + H <= ld)), AQ_E_SHAPE);
  if (B == 0) return AQ_OK;
  SQ_NEED(proj && conv_w && ring && slots && pos && (decay || (dt_bias && a_log)) && state && y);
  SQ_CHECK(!bad_ptr16(state), AQ_E_ALIGN);
  SsdStepArgs a{};
  a.s = ConvSrc{conv_w, conv_b, (int)(H * P + 2 * G * N), (int)taps};
  a.slots = slots, a.pos = pos, a.dt_bias = dt_bias, a.a_log = a_log, a.skip = skip, a.decay = decay, a.state = state, a.y = y;
  a.ld = ld, a.o_xbc = o_xbc, a.o_dt = o_dt;
  a.H = (int)H, a.G = (int)G, a.N = (int)N, a.P = (int)P;
  constexpr int NI = SSD_STEP_COLS / 16;
  SQ_CHECK(H * P < (1 << 24), AQ_E_RANGE);
  const dim3 grid((unsigned)(H * ((P + SSD_STEP_COLS - 1) / SSD_STEP_COLS)), (unsigned)B);
  SQ_DISPATCH(dtype, SQ_ROWS(N, (ssd_step_kernel<T, RP, NI><<<grid, 256, 0, (hipStream_t)stream>>>(a, (const T*)proj, (T*)ring))));
  return launched();
}
