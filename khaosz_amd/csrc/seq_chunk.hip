// The two linear recurrences over long prompts, in chunks of 64 tokens on the fp32 matrix cores
// (v_mfma_f32_16x16x4_f32: every operand and sum stays fp32).  seq_scan.hip does one token after the other; here the
// tokens of a chunk meet in matrix products and only the step from chunk to chunk is sequential.
//
// Delta rule, one head, state S before the chunk, G_i the sum of the chunk's log decays up to and including token i:
//     u_i + beta_i sum_{j<i} <k_i e^{G_i - G_j}, k_j> u_j  =  beta_i (v_i - S^T (k_i e^{G_i}))
//     o_i = S^T (q_i e^{G_i}) + sum_{j<=i} <q_i e^{G_i - G_j}, k_j> u_j
//     S  <- e^{G_C} S + sum_j (k_j e^{G_C - G_j}) u_j^T
// so with (I + A) the unit triangular matrix on the left:  u = U0 - W S  with  W = (I + A)^-1 (beta k e^G),
// U0 = (I + A)^-1 (beta v).  Two launches: `prep` (per chunk and head: convolution, norms, decays, A and the masked
// query-key matrix, W and U0), `scan` (per head and 16 columns of S:
// the chunks in order).
//
// A decay can be anything in (0, 1], so e^{G_i - G_j} must not be split into e^{G_i} and e^{-G_j} across a chunk.  The
// sums are kept by blocks of 16 tokens: between blocks the split point is the later block's start, and both factors are
// at most 1; inside a block it is the block's middle while every factor stays below 2^60, and otherwise the
// differences are exponentiated pair by pair.
//
// State space (SSD), same idea with one scalar decay per head and token: y = e^{L_i} S^T C_i + sum_{j<=i} M_ij x_j + D x_i,
// M_ij = <C_i, B_j> e^{L_i - L_j} dt_j;  S <- e^{L_C} S + sum_j e^{L_C - L_j} dt_j B_j x_j^T.  C B^T belongs to the
// group and is computed once (`ssd_group`), M per head (`ssd_steps`), and the chunks run in order like the delta rule's
// (`ssd_chunks`).  Linear attention with a constant decay per head is the same with dt = 1.
#include "seq_common.h"

namespace sq {

constexpr int CH = 64;    // tokens per chunk
constexpr int BL = 16;    // tokens per block
constexpr int NB = CH / BL;
constexpr int CT = 16;    // state columns per workgroup of the scans
constexpr int MAX_TAPS = 4;
typedef float f32x4 __attribute__((ext_vector_type(4)));

// D[16 x 16] += A[16 x 16] B[16 x 16], contraction in four steps of 4.  Lane l: row (A) or column (B) l % 16, and the
// elements 4 (l / 16) .. + 4 of the contraction; D: column l % 16, rows 4 (l / 16) .. + 4.
__device__ __forceinline__ f32x4 mma16(const float4& a, const float4& b, f32x4 c) {
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, c, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, c, 0, 0, 0);
}
// two of them with their dependent steps interleaved
__device__ __forceinline__ void mma16x2(const float4& a, const float4& b, f32x4& c, const float4& x, const float4& y, f32x4& z) {
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, c, 0, 0, 0);
  z = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, z, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, c, 0, 0, 0);
  z = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, z, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, c, 0, 0, 0);
  z = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, z, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, c, 0, 0, 0);
  z = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, z, 0, 0, 0);
}
__device__ __forceinline__ float ex2(float x) { return __builtin_amdgcn_exp2f(x); }
// The scans read their operands from memory a fragment at a time: 64 lanes x 4 floats of one 16 x 16 block, in lane
// order, so that a load is 1 KB of consecutive memory (rows of a plain matrix would be 16 half-used cache lines).
constexpr int FRAG = 256;
// accumulator layout (column l % 16, rows 4 (l / 16) + r) -> left-operand layout (row l' % 16, columns 4 (l' / 16) + s)
// of the same block: a 4 x 4 transpose inside every quad of lanes; the result belongs to fragment lane frag_lane(l).
__device__ __forceinline__ float quad_xor1(float v) {
  return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xf, 0xf, true));
}
__device__ __forceinline__ float quad_xor2(float v) {
  return __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4E, 0xf, 0xf, true));
}
__device__ __forceinline__ f32x4 quad_transpose(f32x4 v, int lane) {
  const bool o1 = lane & 1, o2 = lane & 2;
  const float a = quad_xor1(o1 ? v[0] : v[1]), b = quad_xor1(o1 ? v[2] : v[3]);
  v = o1 ? f32x4{a, v[1], b, v[3]} : f32x4{v[0], a, v[2], b};
  const float c = quad_xor2(o2 ? v[0] : v[2]), d = quad_xor2(o2 ? v[1] : v[3]);
  return o2 ? f32x4{c, d, v[2], v[3]} : f32x4{v[0], v[1], c, d};
}
__device__ __forceinline__ int frag_lane(int lane) { return ((lane >> 2) & 3) * 16 + (lane >> 4) * 4 + (lane & 3); }
__device__ __forceinline__ float4 ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }

// Convolution + SiLU of one channel over `len` (a multiple of 16) consecutive tokens from token t0 on, of which the
// portion holds n: put(i, value), zero past n.  Inputs are requested 16 at a time at clamped addresses: a load under a
// condition would be waited for where the condition ends.
template <typename T, typename F>
__device__ __forceinline__ void conv_run(const T* in, int64_t ld, int64_t tok0, int t0, int n, int len, int pos, const T* ring,
                                         int taps, int C, int c, const float* w, float bias, F put) {
  float wj[MAX_TAPS], win[MAX_TAPS];  // right-aligned: entry MAX_TAPS - 1 is the current token
  const T* src = in + tok0 * ld + c;
#pragma unroll
  for (int j = 0; j < MAX_TAPS; ++j) {
    const int back = MAX_TAPS - 1 - j;
    wj[j] = back < taps ? w[c * taps + taps - 1 - back] : 0.0f;
    win[j] = 0.0f;
    if (n > 0 && back > 0 && back < taps) {
      const int a = pos + t0 - back;  // position
      if (a >= pos) win[j] = to_f32(src[(int64_t)(a - pos) * ld]);
      else if (a >= 0) win[j] = to_f32(ring[(int64_t)(a % taps) * C + c]);
    }
  }
  const int lastt = n > 0 ? t0 + n - 1 : 0;
  for (int i0 = 0; i0 < len; i0 += 16) {
    T x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) x[i] = src[(int64_t)(i0 + i < n ? t0 + i0 + i : lastt) * ld];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      win[MAX_TAPS - 1] = to_f32(x[i]);
      float acc = bias;
#pragma unroll
      for (int j = 0; j < MAX_TAPS; ++j) acc = fmaf(wj[j], win[j], acc);
#pragma unroll
      for (int j = 0; j + 1 < MAX_TAPS; ++j) win[j] = win[j + 1];
      put(i0 + i, i0 + i < n ? silu(acc) : 0.0f);
    }
  }
}

// ---------------------------------------------------------------------------------------------- delta: prep
struct DeltaChunkArgs {
  const int* slots;
  const int* pos;
  const float* conv_w;   // [C, taps]
  const float* a_log;    // [H]
  const float* dt_bias;  // [H * D]
  // per chunk and head (BC = B * chunks), in fragments of 16 x 16
  float* QK;             // [BC, H, 64 x 64]  left operands
  float* W;              // [BC, H, 64 x DP]  left operands
  float* Q;              // [BC, H, 64 x DP]  q e^G, left operands
  float* K;              // [BC, H, DP x 64]  k e^{G_C - G} transposed, left operands
  float* U;              // [BC, H, 64 x EP]  U0, accumulators
  float* gc;             // [BC, H, DP]      e^{G_C}
  int64_t ld, ld_raw, ld_beta;
  int S, NC, H, G, D, E, DP, EP, taps, C;
};

// block pairs of the chunk's 4 x 4: 0..3 the diagonal, 4..9 below it, 10..15 above
__device__ __forceinline__ void pair_block(int pair, int& I, int& J) {
  constexpr uint64_t ROWS = 0x2101'0033'3221'3210ull, COLS = 0x3332'2121'0100'3210ull;
  I = (int)(ROWS >> (4 * pair)) & 15;
  J = (int)(COLS >> (4 * pair)) & 15;
}

constexpr int PREP_WAVES = 8, PREP_THREADS = 64 * PREP_WAVES;
constexpr int PA = CH + 4, PI = BL + 4, PV = 128 + 4;  // row pitches of A, of the inverted blocks and of v
constexpr int max_of(int a, int b) { return a > b ? a : b; }
// floats of LDS: decays (later A and the inverses), q (later v), k, beta
template <int DP>
struct PrepLds {
  static constexpr int DECAYS = max_of(2 * (CH * (DP + 2) + NB * DP), CH * PA + NB * BL * PI);
  static constexpr int QUERIES = CH * max_of(DP + 4, PV);
  static constexpr int TOTAL = DECAYS + QUERIES + CH * (DP + 4) + CH;
};

template <int DP, typename T>
__global__ __launch_bounds__(PREP_THREADS) void delta_chunk_prep_kernel(DeltaChunkArgs p, const T* qkv, const T* raw, const T* braw, const T* ring0) {
  constexpr int PT = DP + 4, PG = DP + 2;
  extern __shared__ __align__(16) float lds[];
  // log2 decays summed within their block of 16, and the sums of whole blocks.  Only differences of them are used, and
  // one token that forgets everything must not cost the digits of the others: double.
  double* g_s = reinterpret_cast<double*>(lds);  // [64][PG]
  double* tot = g_s + CH * PG;                   // [NB][DP]
  float* q_s = lds + PrepLds<DP>::DECAYS;        // [64][PT], later v
  float* k_s = q_s + PrepLds<DP>::QUERIES;
  float* b_s = k_s + CH * PT;                    // [64] beta
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = blockIdx.x % p.NC, b = blockIdx.x / p.NC, h = blockIdx.y, j = h / (p.H / p.G);
  const int t0 = c * CH, n = p.S - t0 < CH ? p.S - t0 : CH;
  const int pos = p.pos[b], D = p.D, E = p.E;
  const int64_t tok0 = (int64_t)b * p.S, ch = (int64_t)blockIdx.x * p.H + h;
  const T* ring = ring0 + (int64_t)p.slots[b] * p.taps * p.C;

  if (tid < CH) b_s[tid] = tid < n ? sigmoid(to_f32(braw[(tok0 + t0 + tid) * p.ld_beta + h])) : 0.0f;
  for (int x = tid; x < 4 * DP; x += PREP_THREADS) {  // q or k channel, and half of the chunk
    const int y = x % (2 * DP), d = y % DP, i0 = x / (2 * DP) * (CH / 2), m = n - i0 < CH / 2 ? n - i0 : CH / 2;
    float* dst = (y < DP ? q_s : k_s) + i0 * PT + d;
    conv_run(qkv, p.ld, tok0, t0 + i0, d < D && m > 0 ? m : 0, CH / 2, pos, ring, p.taps, p.C,
             (y < DP ? 0 : p.G * D) + j * D + (d < D ? d : D - 1), p.conv_w, 0.0f, [&](int i, float v) { dst[i * PT] = v; });
  }
  const float a = -expf(p.a_log[h]) * 1.44269504088896341f;
  for (int x = tid; x < NB * DP; x += PREP_THREADS) {  // channel and block
    const int d = x % DP, dc = d < D ? d : D - 1, i0 = (x / DP) * BL;
    const float bias = p.dt_bias[h * D + dc];
    const T* src = raw + tok0 * p.ld_raw + h * D + dc;
    T v[BL];
#pragma unroll
    for (int i = 0; i < BL; ++i) v[i] = src[(int64_t)(t0 + (i0 + i < n ? i0 + i : n - 1)) * p.ld_raw];
    double sum = 0.0;
#pragma unroll
    for (int i = 0; i < BL; ++i) {
      const float l = a * softplus_abs(to_f32(v[i]) + bias);
      sum += i0 + i < n && d < D ? (double)l : 0.0;
      g_s[(i0 + i) * PG + d] = sum;
    }
    tot[(i0 / BL) * DP + d] = sum;
  }
  __syncthreads();
  // unit vectors: 16 lanes take a token
  for (int i = wave * 4 + (lane >> 4); i < CH; i += 4 * PREP_WAVES) {
    float sq = 0.0f, sk = 0.0f;
    float* qr = &q_s[i * PT + (lane & 15)];
    float* kr = &k_s[i * PT + (lane & 15)];
#pragma unroll
    for (int d = 0; d < DP; d += 16) sq += qr[d] * qr[d], sk += kr[d] * kr[d];
    const float rq = 1.0f / (sqrtf(row16_sum(sq) + 1e-6f) * sqrtf((float)D)), rk = 1.0f / sqrtf(row16_sum(sk) + 1e-6f);
#pragma unroll
    for (int d = 0; d < DP; d += 16) qr[d] *= rq, kr[d] *= rk;
  }
  __syncthreads();
  const int r16 = lane & 15, q4 = (lane >> 4) * 4;
  // ---- the scaled copies of q and k, a fragment per wavefront and turn
  for (int f = wave; f < NB * (DP / 16); f += PREP_WAVES) {
    {
      const int I = f / (DP / 16), d = (f % (DP / 16)) * 16 + q4, t = I * BL + r16;
      float o[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        double g = g_s[t * PG + d + r];
        for (int k = 0; k < I; ++k) g += tot[k * DP + d + r];
        o[r] = q_s[t * PT + d + r] * ex2((float)g);
      }
      *reinterpret_cast<float4*>(p.Q + ch * CH * DP + f * FRAG + lane * 4) = make_float4(o[0], o[1], o[2], o[3]);
    }
    {
      const int d = (f / NB) * 16 + r16, J = f % NB, t = J * BL + q4;
      double rest = tot[J * DP + d];
      for (int k = J + 1; k < NB; ++k) rest += tot[k * DP + d];
      float o[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = k_s[(t + r) * PT + d] * ex2((float)(rest - g_s[(t + r) * PG + d]));
      *reinterpret_cast<float4*>(p.K + ch * DP * CH + f * FRAG + lane * 4) = make_float4(o[0], o[1], o[2], o[3]);
    }
  }
  for (int d = tid; d < DP; d += PREP_THREADS) p.gc[ch * DP + d] = ex2((float)(tot[d] + tot[DP + d] + tot[2 * DP + d] + tot[3 * DP + d]));
  // ---- A and QK: 10 block pairs I >= J, the four diagonal ones first (one per wavefront)
  constexpr int TURNS = NB * NB / PREP_WAVES;
  f32x4 a_reg[TURNS];  // this wavefront's blocks of A: they go to LDS when q is not needed any more
  float* QK = p.QK + ch * CH * CH;
#pragma unroll
  for (int turn = 0; turn < TURNS; ++turn) {
    const int pair = wave + PREP_WAVES * turn;
    // pairs 0..3: diagonal; 4..9: below it; 10..15: above, zero
    int I, J;
    pair_block(pair, I, J);
    f32x4 sa = {0, 0, 0, 0}, sq = {0, 0, 0, 0};
    const int i = I * BL + r16, jj = J * BL + r16;  // this lane's row (A operand) and column (B operand)
    bool direct = false;
    if (I == J) {
      // both factors around the block's middle; 2^60 leaves room for the sums
      float worst = 0.0f;
      for (int d = q4; d < DP; d += 16)
#pragma unroll
        for (int r = 0; r < 4; ++r) worst = fmaxf(worst, fabsf((float)(g_s[i * PG + d + r] - g_s[(I * BL + BL / 2) * PG + d + r])));
      direct = __builtin_amdgcn_ballot_w64(worst > 60.0f) != 0;
    }
    if (I >= J && !direct) {
      for (int d = q4; d < DP; d += 16) {
        // ei: from the split point to the row; ej: from the column to the split point (the middle of a diagonal block,
        // else the start of the row's block: the rest of the column's block and the blocks between)
        float e_i[4], e_j[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const double gi = g_s[i * PG + d + r], gj = g_s[jj * PG + d + r];
          double to_row = gi, to_split;
          if (I == J) {
            const double mid = g_s[(I * BL + BL / 2) * PG + d + r];
            to_row = gi - mid, to_split = mid - gj;
          } else {
            to_split = tot[J * DP + d + r] - gj;
            for (int k = J + 1; k < I; ++k) to_split += tot[k * DP + d + r];
          }
          e_i[r] = ex2((float)to_row), e_j[r] = ex2((float)to_split);
        }
        const float4 ei = make_float4(e_i[0], e_i[1], e_i[2], e_i[3]), ej = make_float4(e_j[0], e_j[1], e_j[2], e_j[3]);
        const float4 ki = ld4(&k_s[i * PT + d]), qi = ld4(&q_s[i * PT + d]), kj = ld4(&k_s[jj * PT + d]);
        const float4 bj = make_float4(kj.x * ej.x, kj.y * ej.y, kj.z * ej.z, kj.w * ej.w);
        sa = mma16(make_float4(ki.x * ei.x, ki.y * ei.y, ki.z * ei.z, ki.w * ei.w), bj, sa);
        sq = mma16(make_float4(qi.x * ei.x, qi.y * ei.y, qi.z * ei.z, qi.w * ei.w), bj, sq);
      }
    } else if (direct) {
      // entry (row q4 + r, column r16) of the block, pair by pair
      for (int d = 0; d < DP; ++d) {
        const double gj = g_s[jj * PG + d];
        const float kj = k_s[jj * PT + d];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = I * BL + q4 + r;
          const float e = kj * ex2(fminf((float)(g_s[row * PG + d] - gj), 0.0f));  // rows above the diagonal are not used
          sa[r] = fmaf(k_s[row * PT + d], e, sa[r]);
          sq[r] = fmaf(q_s[row * PT + d], e, sq[r]);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = I * BL + q4 + r, col = J * BL + r16;
      a_reg[turn][r] = col < row ? b_s[row] * sa[r] : 0.0f;
      sq[r] = col <= row ? sq[r] : 0.0f;
    }
    *reinterpret_cast<f32x4*>(QK + (I * NB + J) * FRAG + frag_lane(lane) * 4) = quad_transpose(sq, lane);
  }
  // ---- (I + A)^-1 by blocks of 16: X_I = T_I (R_I - sum_{J<I} A_IJ X_J), T_I the inverse of a diagonal block.  A column
  // tile of R in the accumulator layout of mma16 is at the same time its right operand, so a wavefront solves a
  // tile of 16 columns in registers.
  constexpr int WT = (DP / 16 + PREP_WAVES - 1) / PREP_WAVES;  // tiles of W per wavefront
  f32x4 x[WT][NB];
#pragma unroll
  for (int t = 0; t < WT; ++t) {
    const int d = ((wave + PREP_WAVES * t) * 16 + r16) % DP;
    double base = 0.0;
#pragma unroll
    for (int I = 0; I < NB; ++I) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = I * BL + q4 + r;
        x[t][I][r] = b_s[i] * k_s[i * PT + d] * ex2((float)(base + g_s[i * PG + d]));
      }
      base += tot[I * DP + d];
    }
  }
  __syncthreads();  // q, k and the decays are done with
  float* A = reinterpret_cast<float*>(g_s);  // [64][PA]
  float* T_s = A + CH * PA;                  // [NB][16][PI]
#pragma unroll
  for (int turn = 0; turn < TURNS; ++turn) {
    int I, J;
    pair_block(wave + PREP_WAVES * turn, I, J);
#pragma unroll
    for (int r = 0; r < 4; ++r) A[(I * BL + q4 + r) * PA + J * BL + r16] = a_reg[turn][r];
  }
  __syncthreads();
  if (wave == 0) {  // lane: column lane % 16 of block lane / 16
    const float* blk = A + (lane >> 4) * BL * (PA + 1);
    float v[BL];
#pragma unroll
    for (int i = 0; i < BL; ++i) {
      float sum = i == r16 ? 1.0f : 0.0f;
#pragma unroll
      for (int k = 0; k < i; k += 4) {
        const float4 a4 = ld4(&blk[i * PA + k]);
        sum = fmaf(-a4.x, v[k], sum);
        if (k + 1 < i) sum = fmaf(-a4.y, v[k + 1], sum);
        if (k + 2 < i) sum = fmaf(-a4.z, v[k + 2], sum);
        if (k + 3 < i) sum = fmaf(-a4.w, v[k + 3], sum);
      }
      v[i] = sum;
      T_s[((lane >> 4) * BL + i) * PI + r16] = sum;
    }
  }
  // beta v into q's space, 128 channels at a time: thread = (channel, block of 16 tokens)
  float* v_s = q_s;  // [64][PV]
  auto convolve_v = [&](int e0) __attribute__((always_inline)) {
    const int e = e0 + (tid & 127), ec = e < E ? e : E - 1, i0 = (tid >> 7) * BL;
    conv_run(qkv, p.ld, tok0, t0 + i0, e < E ? (n - i0 < BL ? (n - i0 > 0 ? n - i0 : 0) : BL) : 0, BL, pos, ring, p.taps, p.C,
             2 * p.G * D + h * E + ec, p.conv_w, 0.0f, [&](int i, float v) { v_s[(i0 + i) * PV + (tid & 127)] = b_s[i0 + i] * v; });
  };
  convolve_v(0);
  __syncthreads();
  float4 am[NB][NB], tm[NB];
#pragma unroll
  for (int I = 0; I < NB; ++I) {
    tm[I] = ld4(&T_s[(I * BL + r16) * PI + q4]);
#pragma unroll
    for (int J = 0; J < I; ++J) {
      am[I][J] = ld4(&A[(I * BL + r16) * PA + J * BL + q4]);
      am[I][J] = make_float4(-am[I][J].x, -am[I][J].y, -am[I][J].z, -am[I][J].w);
    }
  }
  auto solve = [&](f32x4 (&y)[NB]) __attribute__((always_inline)) {
#pragma unroll
    for (int I = 0; I < NB; ++I) {
#pragma unroll
      for (int J = 0; J < I; ++J) y[I] = mma16(am[I][J], make_float4(y[J][0], y[J][1], y[J][2], y[J][3]), y[I]);
      y[I] = mma16(tm[I], make_float4(y[I][0], y[I][1], y[I][2], y[I][3]), f32x4{0, 0, 0, 0});
    }
  };
#pragma unroll
  for (int t = 0; t < WT; ++t) {
    if ((wave + PREP_WAVES * t) * 16 >= DP) break;
    solve(x[t]);
#pragma unroll
    for (int I = 0; I < NB; ++I)
      *reinterpret_cast<f32x4*>(p.W + ch * CH * DP + (I * (DP / 16) + wave + PREP_WAVES * t) * FRAG + frag_lane(lane) * 4) = quad_transpose(x[t][I], lane);
  }
  for (int e0 = 0; e0 < p.EP; e0 += 128) {
    if (e0) {
      __syncthreads();
      convolve_v(e0);
      __syncthreads();
    }
    if (e0 + wave * 16 >= p.EP) continue;
    f32x4 y[NB];
#pragma unroll
    for (int I = 0; I < NB; ++I)
#pragma unroll
      for (int r = 0; r < 4; ++r) y[I][r] = v_s[(I * BL + q4 + r) * PV + wave * 16 + r16];
    solve(y);
#pragma unroll
    for (int I = 0; I < NB; ++I)
      *reinterpret_cast<f32x4*>(p.U + ch * CH * p.EP + (I * (p.EP / 16) + e0 / 16 + wave) * FRAG + lane * 4) = y[I];
  }
}

// ---------------------------------------------------------------------------------------------- delta: scan
struct DeltaScanArgs {
  const float *W, *U, *Q, *K, *QK, *gc;
  float* state;  // [slots, H, E, D]
  float* out;    // [M, H, E]
  const int* slots;
  const int* pos;
  int S, NC, H, D, E, EP;
};

// rows d .. d + 4 of a state column (rows past D are zero)
__device__ __forceinline__ f32x4 load_state4(const float* col, int d, int D, bool ok) {
  f32x4 v = {0, 0, 0, 0};
  if (!ok) return v;
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (d + r < D) v[r] = col[d + r];
  return v;
}
__device__ __forceinline__ void store_state4(float* col, int d, int D, const f32x4& v) {
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (d + r < D) col[d + r] = v[r];
}

template <int DP>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 1))) void delta_chunk_scan_kernel(DeltaScanArgs p) {
  constexpr int KB = DP / 16;               // groups of 16 in the contraction over rows
  constexpr int NT = (KB + 3) / 4;          // 16-row tiles of the state per wavefront
  constexpr int SP = DP + 4, UP = CH + 4;
  __shared__ __align__(16) float s_s[CT * SP];  // the state, column by column
  __shared__ __align__(16) float u_s[CT * UP];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r16 = lane & 15, q4 = (lane >> 4) * 4;
  // heads first: the tiles of a head read the same chunks, and workgroups go round robin over the XCDs and their caches
  const int tile = blockIdx.y, h = blockIdx.x, b = blockIdx.z;
  const int e = tile * CT + r16, D = p.D;
  float* col = p.state + (((int64_t)p.slots[b] * p.H + h) * p.E + (e < p.E ? e : 0)) * D;
  f32x4 s[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int d = (wave + 4 * t) * 16 + q4;
    s[t] = load_state4(col, d, D, e < p.E && p.pos[b] > 0 && d < DP);
  }
  // everything a chunk brings, in registers; the next chunk's is requested before this one's work begins
  struct Chunk {
    float4 w[KB], q[KB], k[NT][NB], a[NB], gc[NT];
    f32x4 u0;
  };
  Chunk c0, c1;
  auto index = [&](int c) -> int64_t { return ((int64_t)b * p.NC + (c < p.NC ? c : p.NC - 1)) * p.H + h; };
  auto load_wq = [&](Chunk& r, int64_t ch, int x) __attribute__((always_inline)) {
      r.w[x] = ld4(p.W + ch * CH * DP + (wave * KB + x) * FRAG + lane * 4);
      r.q[x] = ld4(p.Q + ch * CH * DP + (wave * KB + x) * FRAG + lane * 4);
  };
  const int dt[2] = {KB >= 4 || wave < KB ? wave : 0, wave + 4};  // wavefronts without a tile read another's
  auto load_ak = [&](Chunk& r, int64_t ch, int x) __attribute__((always_inline)) {
    r.a[x] = ld4(p.QK + ch * CH * CH + (wave * NB + x) * FRAG + lane * 4);
#pragma unroll
    for (int t = 0; t < NT; ++t) r.k[t][x] = ld4(p.K + ch * DP * CH + (dt[t] * NB + x) * FRAG + lane * 4);
  };
  auto load_rest = [&](Chunk& r, int64_t ch) __attribute__((always_inline)) {
#pragma unroll
    for (int t = 0; t < NT; ++t) r.gc[t] = ld4(p.gc + ch * DP + dt[t] * 16 + q4);
    r.u0 = *reinterpret_cast<const f32x4*>(p.U + ch * CH * p.EP + (wave * (p.EP / 16) + tile) * FRAG + lane * 4);
  };
  auto chunk = [&](const Chunk& r, Chunk& next, int c) __attribute__((always_inline)) {
#pragma unroll
    for (int t = 0; t < NT; ++t)
      if (wave + 4 * t < KB) *reinterpret_cast<f32x4*>(&s_s[r16 * SP + (wave + 4 * t) * 16 + q4]) = s[t];
    const int64_t nx = index(c + 1);
    __syncthreads();
    f32x4 ws = {0, 0, 0, 0}, o = {0, 0, 0, 0};
    float4 sv[KB];
#pragma unroll
    for (int x = 0; x < KB; ++x) sv[x] = ld4(&s_s[r16 * SP + x * 16 + q4]);
#pragma unroll
    for (int x = 0; x < KB; ++x) {  // loads between the products: in a row they would hold up the wavefronts
      mma16x2(r.w[x], sv[x], ws, r.q[x], sv[x], o);
      load_wq(next, nx, x);
      __builtin_amdgcn_sched_barrier(0);
    }
    const f32x4 u = r.u0 - ws;
    *reinterpret_cast<f32x4*>(&u_s[r16 * UP + wave * BL + q4]) = u;
    __syncthreads();
    float4 uv[NB];
#pragma unroll
    for (int x = 0; x < NB; ++x) uv[x] = ld4(&u_s[r16 * UP + x * 16 + q4]);
#pragma unroll
    for (int t = 0; t < NT; ++t) s[t][0] *= r.gc[t].x, s[t][1] *= r.gc[t].y, s[t][2] *= r.gc[t].z, s[t][3] *= r.gc[t].w;
#pragma unroll
    for (int x = 0; x < NB; ++x) {
      mma16x2(r.a[x], uv[x], o, r.k[0][x], uv[x], s[0]);
#pragma unroll
      for (int t = 1; t < NT; ++t) s[t] = mma16(r.k[t][x], uv[x], s[t]);
      load_ak(next, nx, x);
      __builtin_amdgcn_sched_barrier(0);
    }
    load_rest(next, nx);
    const int t0 = c * CH + wave * BL + q4;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (t0 + i < p.S && e < p.E) p.out[(((int64_t)b * p.S + t0 + i) * p.H + h) * p.E + e] = o[i];
  };
#pragma unroll
  for (int x = 0; x < KB; ++x) load_wq(c0, index(0), x);
#pragma unroll
  for (int x = 0; x < NB; ++x) load_ak(c0, index(0), x);
  load_rest(c0, index(0));
  for (int c = 0; c < p.NC; c += 2) {
    chunk(c0, c1, c);
    if (c + 1 < p.NC) chunk(c1, c0, c + 1);
  }
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int d = (wave + 4 * t) * 16 + q4;
    if (e < p.E && d < DP) store_state4(col, d, D, s[t]);
  }
}

// ---------------------------------------------------------------------------------------------- state space
struct SsdChunkArgs {
  const int* slots;
  const int* pos;
  const float* conv_w;  // [C, taps], channels x | B | C
  const float* conv_b;
  const float* dt_bias;
  const float* a_log;
  const float* skip;    // or null
  const float* decay;   // [H] constant decays (step size 1), or null
  // per chunk and group, left operands in fragments of 16 x 16
  float* CB;     // [BC, G, 64 x 64]
  float* Cm;     // [BC, G, 64 x NP]
  float* Bt;     // [BC, G, NP x 64]  B transposed
  // per chunk and head
  float* Mx;     // [BC, H, 64 x 64]  <C_i, B_j> e^{L_i - L_j} dt_j, left operands (blocks above the diagonal are not written)
  float* el;     // [BC, H, 64]  e^{L_i}
  float* wj;     // [BC, H, 64]  dt_j e^{L_C - L_j}
  float* dc;     // [BC, H]      e^{L_C}
  float* state;  // [slots, H, P, N]
  float* out;    // [M, H, P]
  int64_t ld, ld_dt;
  int S, NC, H, G, N, P, NP, taps, C;
};

template <int NP, typename T>
__global__ __launch_bounds__(256) void ssd_group_kernel(SsdChunkArgs p, const T* xbc, const T* ring0) {
  constexpr int PT = NP + 4;
  extern __shared__ __align__(16) float lds[];
  float* b_s = lds;            // [64][PT]
  float* c_s = lds + CH * PT;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = blockIdx.x % p.NC, b = blockIdx.x / p.NC, g = blockIdx.y;
  const int t0 = c * CH, n = p.S - t0 < CH ? p.S - t0 : CH, pos = p.pos[b], N = p.N;
  const int64_t tok0 = (int64_t)b * p.S, ch = (int64_t)blockIdx.x * p.G + g;
  const T* ring = ring0 + (int64_t)p.slots[b] * p.taps * p.C;
  for (int x = tid; x < 2 * NP * NB; x += 256) {  // channel and block of 16 tokens
    const int y = x % (2 * NP), d = y % NP, i0 = (x / (2 * NP)) * BL;
    float* dst = (y < NP ? b_s : c_s) + i0 * PT + d;
    const int m = d < N ? (n - i0 < BL ? (n - i0 > 0 ? n - i0 : 0) : BL) : 0;
    const int chan = p.H * p.P + (y < NP ? 0 : p.G * N) + g * N + (d < N ? d : N - 1);
    conv_run(xbc, p.ld, tok0, t0 + i0, m, BL, pos, ring, p.taps, p.C, chan, p.conv_w, p.conv_b[chan],
             [&](int i, float v) { dst[i * PT] = v; });
  }
  __syncthreads();
  const int r16 = lane & 15, q4 = (lane >> 4) * 4;
  for (int f = wave; f < NB * (NP / 16); f += 4) {
    const int I = f / (NP / 16), d = (f % (NP / 16)) * 16 + q4;
    *reinterpret_cast<float4*>(p.Cm + ch * CH * NP + f * FRAG + lane * 4) = ld4(&c_s[(I * BL + r16) * PT + d]);
    const float* src = &b_s[((f % NB) * BL + q4) * PT + (f / NB) * 16 + r16];
    *reinterpret_cast<float4*>(p.Bt + ch * NP * CH + f * FRAG + lane * 4) = make_float4(src[0], src[PT], src[2 * PT], src[3 * PT]);
  }
  for (int J = 0; J < NB; ++J) {
    f32x4 s = {0, 0, 0, 0};
    if (J <= wave)
      for (int d = q4; d < NP; d += 16) s = mma16(ld4(&c_s[(wave * BL + r16) * PT + d]), ld4(&b_s[(J * BL + r16) * PT + d]), s);
    *reinterpret_cast<f32x4*>(p.CB + ch * CH * CH + (wave * NB + J) * FRAG + frag_lane(lane) * 4) = quad_transpose(s, lane);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void ssd_steps_kernel(SsdChunkArgs p, const T* dt_raw) {
  __shared__ double l_s[CH];  // log2 decays summed from the chunk's start; differences of them are exponentiated
  __shared__ __align__(16) float dt_s[CH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = blockIdx.x % p.NC, b = blockIdx.x / p.NC, h = blockIdx.y, g = h / (p.H / p.G);
  const int64_t ch = (int64_t)blockIdx.x * p.H + h, cg = (int64_t)blockIdx.x * p.G + g;
  if (wave == 0) {
    const int t = c * CH + lane;
    float dt;
    double L;
    if (p.decay) {
      dt = t < p.S ? 1.0f : 0.0f;
      L = log2(fmax((double)p.decay[h], 1e-300)) * (double)dt;
    } else {
      const float raw = to_f32(dt_raw[((int64_t)b * p.S + (t < p.S ? t : p.S - 1)) * p.ld_dt + h]);
      dt = t < p.S ? softplus(raw + p.dt_bias[h]) : 0.0f;
      L = (double)(-expf(p.a_log[h]) * 1.44269504088896341f) * (double)dt;
    }
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double v = __shfl_up(L, o, 64);
      if (lane >= o) L += v;
    }
    const double LC = __shfl(L, 63, 64);
    l_s[lane] = L;
    dt_s[lane] = dt;
    p.el[ch * CH + lane] = ex2((float)L);
    p.wj[ch * CH + lane] = dt * ex2((float)(LC - L));
    if (lane == 0) p.dc[ch] = ex2((float)LC);
  }
  __syncthreads();
  const int row = wave * BL + (lane & 15), q4 = (lane >> 4) * 4;
  const double Li = l_s[row];
  for (int J = 0; J <= wave; ++J) {
    const float4 cb = ld4(p.CB + cg * CH * CH + (wave * NB + J) * FRAG + lane * 4);
    float m[4] = {cb.x, cb.y, cb.z, cb.w};
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = J * BL + q4 + r;
      m[r] = j <= row ? m[r] * dt_s[j] * ex2((float)(Li - l_s[j])) : 0.0f;
    }
    *reinterpret_cast<float4*>(p.Mx + ch * CH * CH + (wave * NB + J) * FRAG + lane * 4) = make_float4(m[0], m[1], m[2], m[3]);
  }
}

template <int NP, typename T>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 1))) void ssd_chunks_kernel(SsdChunkArgs p, const T* xbc,
                                                                                                    const T* ring0) {
  constexpr int KB = NP / 16, NT = (KB + 3) / 4, SP = NP + 4, XP = CH + 4;
  __shared__ __align__(16) float s_s[CT * SP];
  __shared__ __align__(16) float x_s[2][CT * XP];  // the chunk's x, column by column
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r16 = lane & 15, q4 = (lane >> 4) * 4;
  const int tile = blockIdx.y, h = blockIdx.x, b = blockIdx.z, g = h / (p.H / p.G);
  const int e = tile * CT + r16, N = p.N, P = p.P, pos = p.pos[b];
  const int64_t tok0 = (int64_t)b * p.S;
  const T* ring = ring0 + (int64_t)p.slots[b] * p.taps * p.C;
  float* col = p.state + (((int64_t)p.slots[b] * p.H + h) * P + (e < P ? e : 0)) * N;
  f32x4 s[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int d = (wave + 4 * t) * 16 + q4;
    s[t] = load_state4(col, d, N, e < P && pos > 0 && d < NP);
  }
  const float skip = p.skip ? p.skip[h] : 0.0f;
  // x: thread = (column tid % 16, tokens 4 (tid / 16) .. + 4); its raw inputs are requested a chunk ahead
  const int xe = tid & 15, xt = (tid >> 4) * 4;
  const bool xok = tile * CT + xe < P;
  const int xc = h * P + (xok ? tile * CT + xe : P - 1);
  float wj[MAX_TAPS];
  // what a chunk brings, in registers; the next chunk's is requested before this one's work begins.  x as
  // loaded: a conversion here would wait for the load.
  struct Chunk {
    float4 cm[KB], m[NB], bt[NT][NB], w[NB], el;
    T xin[4 + MAX_TAPS - 1];
    float dc;
  };
  Chunk c0, c1;
#pragma unroll
  for (int j = 0; j < MAX_TAPS; ++j) {
    const int back = MAX_TAPS - 1 - j;
    wj[j] = xok && back < p.taps ? p.conv_w[xc * p.taps + p.taps - 1 - back] : 0.0f;
  }
  const float xb = xok ? p.conv_b[xc] : 0.0f;
  auto index = [&](int c) -> int64_t { return ((int64_t)b * p.NC + (c < p.NC ? c : p.NC - 1)) * p.G + g; };
  auto load_x = [&](Chunk& q, int c) __attribute__((always_inline)) {
    if (c >= p.NC) c = p.NC - 1;
#pragma unroll
    for (int i = 0; i < 4 + MAX_TAPS - 1; ++i) {
      const int t = c * CH + xt + i - (MAX_TAPS - 1), tc = t < 0 ? 0 : t < p.S ? t : p.S - 1;
      q.xin[i] = xbc[(tok0 + tc) * p.ld + xc];
    }
    const int64_t chh = ((int64_t)b * p.NC + c) * p.H + h;
    q.el = ld4(p.el + chh * CH + wave * BL + q4);
    q.dc = p.dc[chh];
  };
  auto load_c = [&](Chunk& q, int64_t ch, int x) __attribute__((always_inline)) {
    q.cm[x] = ld4(p.Cm + ch * CH * NP + (wave * KB + x) * FRAG + lane * 4);
  };
  const int dt4[2] = {KB >= 4 || wave < KB ? wave : 0, wave + 4};  // wavefronts without a tile read another's
  auto load_b = [&](Chunk& q, int64_t ch, int x) __attribute__((always_inline)) {
    const int64_t chh = ch / p.G * p.H + h;
    q.m[x] = ld4(p.Mx + chh * CH * CH + (wave * NB + x) * FRAG + lane * 4);
    q.w[x] = ld4(p.wj + chh * CH + x * 16 + q4);
#pragma unroll
    for (int t = 0; t < NT; ++t) q.bt[t][x] = ld4(p.Bt + ch * NP * CH + (dt4[t] * NB + x) * FRAG + lane * 4);
  };
  load_x(c0, 0);
#pragma unroll
  for (int x = 0; x < KB; ++x) load_c(c0, index(0), x);
#pragma unroll
  for (int x = 0; x < NB; ++x) load_b(c0, index(0), x);
#pragma unroll
  for (int i = 0; i < MAX_TAPS - 1; ++i) {  // inputs from before the portion
    const int t = xt + i - (MAX_TAPS - 1), a = pos + t;
    if (t < 0) c0.xin[i] = a >= 0 && t > -p.taps ? ring[(int64_t)(a % p.taps) * p.C + xc] : from_f32<T>(0.0f);
  }
  auto chunk = [&](const Chunk& q, Chunk& next, int c) __attribute__((always_inline)) {
    const int buf = c & 1;
    // ---- this chunk's x; the state as an operand
    float4 xv;
    {
      float y[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float acc = xb;
#pragma unroll
        for (int j = 0; j < MAX_TAPS; ++j) acc = fmaf(wj[j], to_f32(q.xin[i + j]), acc);
        y[i] = xok && c * CH + xt + i < p.S ? silu(acc) : 0.0f;
      }
      xv = make_float4(y[0], y[1], y[2], y[3]);
    }
    *reinterpret_cast<float4*>(&x_s[buf][xe * XP + xt]) = xv;
#pragma unroll
    for (int t = 0; t < NT; ++t)
      if (wave + 4 * t < KB) *reinterpret_cast<f32x4*>(&s_s[r16 * SP + (wave + 4 * t) * 16 + q4]) = s[t];
    const int64_t nx = index(c + 1);
    __syncthreads();
    f32x4 y = {0, 0, 0, 0}, y1 = {0, 0, 0, 0};
    float4 sv[KB];
#pragma unroll
    for (int x = 0; x < KB; ++x) sv[x] = ld4(&s_s[r16 * SP + x * 16 + q4]);
#pragma unroll
    for (int x = 0; x < KB; x += 2) {  // loads between the products: in a row they would hold up the wavefronts
      mma16x2(q.cm[x], sv[x], y, q.cm[x + 1], sv[x + 1], y1);
      load_c(next, nx, x);
      load_c(next, nx, x + 1);
      __builtin_amdgcn_sched_barrier(0);
    }
    load_x(next, c + 1);
    y += y1;
    __syncthreads();  // the state may be overwritten
    float4 xx[NB];
#pragma unroll
    for (int x = 0; x < NB; ++x) xx[x] = ld4(&x_s[buf][r16 * XP + x * 16 + q4]);
    y[0] *= q.el.x, y[1] *= q.el.y, y[2] *= q.el.z, y[3] *= q.el.w;  // tokens wave * 16 + q4 + r
#pragma unroll
    for (int x = 0; x < NB; ++x) {
      if (x > wave) break;  // keys ahead of every token of the wavefront
      y = mma16(q.m[x], xx[x], y);
    }
#pragma unroll
    for (int x = 0; x < NB; ++x) {
      const float4 wv = q.w[x];
      const float4 xw = make_float4(xx[x].x * wv.x, xx[x].y * wv.y, xx[x].z * wv.z, xx[x].w * wv.w);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        if (x == 0) s[t] *= q.dc;
        s[t] = mma16(q.bt[t][x], xw, s[t]);
      }
      load_b(next, nx, x);
      __builtin_amdgcn_sched_barrier(0);
    }
    const int t0 = c * CH + wave * BL + q4;
    const float4 own = ld4(&x_s[buf][r16 * XP + wave * BL + q4]);
    const float xo[4] = {own.x, own.y, own.z, own.w};
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (t0 + r < p.S && e < P) p.out[(((int64_t)b * p.S + t0 + r) * p.H + h) * P + e] = y[r] + skip * xo[r];
  };
  for (int c = 0; c < p.NC; c += 2) {
    chunk(c0, c1, c);
    if (c + 1 < p.NC) chunk(c1, c0, c + 1);
  }
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int d = (wave + 4 * t) * 16 + q4;
    if (e < P && d < NP) store_state4(col, d, N, s[t]);
  }
}

inline int64_t pad_rows(int64_t n) { return n <= 32 ? 32 : n <= 64 ? 64 : 128; }
inline int64_t pad16(int64_t n) { return (n + 15) / 16 * 16; }

}  // namespace sq

using namespace sq;

#define SQ_PADDED(R, ...)            \
  do {                               \
    if ((R) <= 32) {                 \
      constexpr int RP = 32;         \
      __VA_ARGS__;                   \
    } else if ((R) <= 64) {          \
      constexpr int RP = 64;         \
      __VA_ARGS__;                   \
    } else {                         \
      constexpr int RP = 128;        \
      __VA_ARGS__;                   \
    }                                \
  } while (0)

template <typename K>
static int big_lds(K* kernel, size_t bytes) {
  if (bytes <= 64 * 1024) return 0;
  return (int)hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
}

extern "C" int aqs_chunked_ok(int64_t rows, int64_t taps) { return rows > 0 && rows <= 128 && taps > 0 && taps <= MAX_TAPS; }

// floats of workspace for B sequences of S tokens
extern "C" int64_t aqs_delta_chunked_ws(int64_t B, int64_t S, int64_t H, int64_t D, int64_t E) {
  const int64_t DP = pad_rows(D), EP = pad16(E);
  return B * ((S + CH - 1) / CH) * H * (CH * CH + 3 * CH * DP + CH * EP + DP);
}
extern "C" int64_t aqs_ssd_chunked_ws(int64_t B, int64_t S, int64_t H, int64_t G, int64_t N) {
  const int64_t NP = pad_rows(N);
  return B * ((S + CH - 1) / CH) * (G * (CH * CH + 2 * CH * NP) + H * (CH * CH + 2 * CH + 1));
}

extern "C" int aqs_delta_chunked(const void* qkv, int64_t ld, const void* raw, int64_t ld_raw, const void* beta_raw, int64_t ld_beta,
                                 int dtype, const float* w, const void* ring, const int32_t* slots, const int32_t* pos,
                                 const float* a_log, const float* dt_bias, float* ws, int64_t ws_floats, float* state, float* out,
                                 int64_t B, int64_t S, int64_t H, int64_t G, int64_t D, int64_t E, int64_t taps, void* stream) {
  SQ_CHECK(B >= 0 && S >= 0 && H > 0 && G > 0 && H % G == 0 && D > 0 && E > 0 && aqs_chunked_ok(D, taps), AQ_E_SHAPE);
  SQ_CHECK(ld >= 2 * G * D + H * E && ld_raw >= H * D && ld_beta >= H, AQ_E_SHAPE);
  const int64_t NC = (S + CH - 1) / CH;
  SQ_CHECK(B * NC < (1 << 16) && H < 65536 && B < 65536 && E <= (1 << 16), AQ_E_RANGE);
  if (B * S == 0) return AQ_OK;
  SQ_NEED(qkv && raw && beta_raw && w && ring && slots && pos && a_log && dt_bias && ws && state && out);
  SQ_CHECK(!bad_ptr16(ws), AQ_E_ALIGN);
  SQ_CHECK(ws_floats >= aqs_delta_chunked_ws(B, S, H, D, E), AQ_E_WORKSPACE);
  const int64_t DP = pad_rows(D), EP = pad16(E), n = B * NC * H;
  DeltaChunkArgs a{};
  a.slots = slots, a.pos = pos, a.conv_w = w, a.a_log = a_log, a.dt_bias = dt_bias;
  a.QK = ws;
  a.W = a.QK + n * CH * CH;
  a.Q = a.W + n * CH * DP;
  a.K = a.Q + n * CH * DP;
  a.U = a.K + n * CH * DP;
  a.gc = a.U + n * CH * EP;
  a.ld = ld, a.ld_raw = ld_raw, a.ld_beta = ld_beta;
  a.S = (int)S, a.NC = (int)NC, a.H = (int)H, a.G = (int)G, a.D = (int)D, a.E = (int)E, a.DP = (int)DP, a.EP = (int)EP;
  a.taps = (int)taps, a.C = (int)(2 * G * D + H * E);
  hipStream_t st = (hipStream_t)stream;
  SQ_DISPATCH(dtype, SQ_PADDED(D, {
                constexpr size_t lds = PrepLds<RP>::TOTAL * sizeof(float);
                if (const int rc = big_lds(&delta_chunk_prep_kernel<RP, T>, lds)) return rc;
                (delta_chunk_prep_kernel<RP, T><<<dim3((unsigned)(B * NC), (unsigned)H), PREP_THREADS, lds, st>>>(
                    a, (const T*)qkv, (const T*)raw, (const T*)beta_raw, (const T*)ring));
              }));
  if (const int rc = launched()) return rc;
  const DeltaScanArgs s{a.W, a.U, a.Q, a.K, a.QK, a.gc, state, out, slots, pos, (int)S, (int)NC, (int)H, (int)D, (int)E, (int)EP};
  const dim3 grid((unsigned)H, (unsigned)(EP / CT), (unsigned)B);
  SQ_PADDED(D, (delta_chunk_scan_kernel<RP><<<grid, 256, 0, st>>>(s)));
  return launched();
}

extern "C" int aqs_ssd_chunked(const void* xbc, int64_t ld, const void* dt_raw, int64_t ld_dt, int dtype, const float* conv_w,
                               const float* conv_b, const void* ring, const int32_t* slots, const int32_t* pos, const float* dt_bias,
                               const float* a_log, const float* skip, const float* decay, float* ws, int64_t ws_floats, float* state,
                               float* out, int64_t B, int64_t S, int64_t H, int64_t G, int64_t N, int64_t P, int64_t taps, void* stream) {
  SQ_CHECK(B >= 0 && S >= 0 && H > 0 && G > 0 && H % G == 0 && N > 0 && P > 0 && aqs_chunked_ok(N, taps), AQ_E_SHAPE);
  SQ_CHECK(ld >= H * P + 2 * G * N && (decay || ld_dt >= H), AQ_E_SHAPE);
  const int64_t NC = (S + CH - 1) / CH;
  SQ_CHECK(B * NC < (1 << 16) && H < 65536 && G < 65536 && B < 65536 && P <= (1 << 16), AQ_E_RANGE);
  if (B * S == 0) return AQ_OK;
  SQ_NEED(xbc && conv_w && conv_b && ring && slots && pos && (decay || (dt_raw && dt_bias && a_log)) && ws && state && out);
  SQ_CHECK(!bad_ptr16(ws), AQ_E_ALIGN);
  SQ_CHECK(ws_floats >= aqs_ssd_chunked_ws(B, S, H, G, N), AQ_E_WORKSPACE);
  const int64_t NP = pad_rows(N), n = B * NC * G;
  SsdChunkArgs a{};
  a.slots = slots, a.pos = pos, a.conv_w = conv_w, a.conv_b = conv_b, a.dt_bias = dt_bias, a.a_log = a_log;
  a.skip = skip, a.decay = decay;
  a.CB = ws;
  a.Cm = a.CB + n * CH * CH;
  a.Bt = a.Cm + n * CH * NP;
  a.Mx = a.Bt + n * CH * NP;
  a.el = a.Mx + B * NC * H * CH * CH;
  a.wj = a.el + B * NC * H * CH;
  a.dc = a.wj + B * NC * H * CH;
  a.state = state, a.out = out, a.ld = ld, a.ld_dt = ld_dt;
  a.S = (int)S, a.NC = (int)NC, a.H = (int)H, a.G = (int)G, a.N = (int)N, a.P = (int)P, a.NP = (int)NP;
  a.taps = (int)taps, a.C = (int)(H * P + 2 * G * N);
  hipStream_t st = (hipStream_t)stream;
  const size_t lds = (size_t)(2 * CH * (NP + 4)) * 4;
  SQ_DISPATCH(dtype, SQ_PADDED(N, {
                if (const int rc = big_lds(&ssd_group_kernel<RP, T>, lds)) return rc;
                (ssd_group_kernel<RP, T><<<dim3((unsigned)(B * NC), (unsigned)G), 256, lds, st>>>(a, (const T*)xbc, (const T*)ring));
              }));
  if (const int rc = launched()) return rc;
  const dim3 grid((unsigned)H, (unsigned)((P + CT - 1) / CT), (unsigned)B);
  SQ_DISPATCH(dtype, (ssd_steps_kernel<T><<<dim3((unsigned)(B * NC), (unsigned)H), 256, 0, st>>>(a, (const T*)dt_raw)));
  if (const int rc = launched()) return rc;
  SQ_DISPATCH(dtype, SQ_PADDED(N, (ssd_chunks_kernel<RP, T><<<grid, 256, 0, st>>>(a, (const T*)xbc, (const T*)ring))));
  return launched();
}
