// Routed feed-forwards: every token goes through the `top` experts with the largest scores sigmoid(<router, h>), each on
// the token scaled by its score (the scale is applied to the expert's two input products, in fp32).
//
// Prompts: `route` (scores and choice), `sort` (tokens by expert, and a list of row tiles), two grouped products over the
// tiles -- gate and up with the GLU behind, then down --; the row operation that adds the feed-forward to the residual
// stream collects a token's rows.  Steps of a few tokens: two launches that read the chosen experts' weights row by row;
// the second adds the chosen experts and the shared one.
#include "seq_common.h"

namespace sq {

constexpr int MAX_EXPERTS = 512, EPL = MAX_EXPERTS / 16;  // scores per lane of a row of 16 lanes

// (value, index) maximum over a row of 16 lanes, in all of them; equal values: the lower index
template <int CTRL>
__device__ __forceinline__ void max_step(float& v, int& i) {
  const float ov = __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), CTRL, 0xf, 0xf, true));
  const int oi = __builtin_amdgcn_mov_dpp(i, CTRL, 0xf, 0xf, true);
  const bool take = ov > v || (ov == v && oi < i);
  v = take ? ov : v;
  i = take ? oi : i;
}
__device__ __forceinline__ void row16_argmax(float& v, int& i) {
  max_step<0xB1>(v, i);
  max_step<0x4E>(v, i);
  max_step<0x141>(v, i);
  max_step<0x140>(v, i);
}
// The `top` largest of Ex scores in z (fp32, anywhere), by a row of 16 lanes: emit(j, expert, score) in all of them.
// NE: scores per lane.
template <int NE, typename F>
__device__ __forceinline__ void choose(const float* z, int Ex, int top, int l16, F emit) {
  float s[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = i * 16 + l16;
    const float v = z[e < Ex ? e : 0];
    s[i] = e < Ex ? v : -INFINITY;
  }
  for (int j = 0; j < top; ++j) {
    float v = s[0];
    int at = l16;
#pragma unroll
    for (int i = 1; i < NE; ++i) {
      const bool take = s[i] > v;
      v = take ? s[i] : v;
      at = take ? i * 16 + l16 : at;
    }
    row16_argmax(v, at);
    at = at < Ex ? at : Ex - 1;
    emit(j, at, v);
#pragma unroll
    for (int i = 0; i < NE; ++i) s[i] = at == i * 16 + l16 ? -INFINITY : s[i];
  }
}
template <typename F>
__device__ __forceinline__ void choose_any(const float* z, int Ex, int top, int l16, F emit) {
  if (Ex <= 64) choose<4>(z, Ex, top, l16, emit);
  else if (Ex <= 128) choose<8>(z, Ex, top, l16, emit);
  else choose<EPL>(z, Ex, top, l16, emit);
}

// ---------------------------------------------------------------------------------------------- prompts: routing
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

struct RouteArgs {
  int* ids;       // [M, top]
  float* scores;  // [M, top]
  int64_t ldh;
  int M, K, Ex, top;
};

// any type and size: a wavefront per token, four experts at a time
template <typename T>
__global__ __launch_bounds__(256) void route_any_kernel(RouteArgs p, const T* h, const T* w) {
  __shared__ float z_s[4][MAX_EXPERTS];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t m = (int64_t)blockIdx.x * 4 + wave;
  if (m >= p.M) return;
  const T* hr = h + m * p.ldh;
  for (int e0 = 0; e0 < p.Ex; e0 += 4) {
    float acc[4] = {0, 0, 0, 0};
    const T* wr[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) wr[i] = w + (int64_t)(e0 + i < p.Ex ? e0 + i : 0) * p.K;
    for (int k = lane; k < p.K; k += 64) {
      const float x = to_f32(hr[k]);
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] = fmaf(x, to_f32(wr[i][k]), acc[i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float s = wave_sum(acc[i]);
      if (lane == 0 && e0 + i < p.Ex) z_s[wave][e0 + i] = s;
    }
  }
  __builtin_amdgcn_wave_barrier();
  choose_any(z_s[wave], p.Ex, p.top, lane & 15, [&](int j, int e, float z) {
    if (lane == 0) {
      p.ids[m * p.top + j] = e;
      p.scores[m * p.top + j] = sigmoid(z);
    }
  });
}

// bf16 on the matrix cores: 16 tokens per workgroup, every wavefront all experts over a quarter of the contraction (steps
// of 32 in turn).  NT: tiles of 16 experts.
template <int NT>
__global__ __launch_bounds__(256) void route_mfma_kernel(RouteArgs p, const uint16_t* h, const uint16_t* w) {
  constexpr int ZP = NT * 16 + 4;
  __shared__ __align__(16) float z_s[4][16][ZP];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, q = lane >> 4;
  const int64_t m0 = (int64_t)blockIdx.x * 16;
  const uint16_t* hr = h + (m0 + r16 < p.M ? m0 + r16 : p.M - 1) * p.ldh;
  const uint16_t* wr[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) wr[t] = w + (int64_t)(t * 16 + r16 < p.Ex ? t * 16 + r16 : p.Ex - 1) * p.K;
  f32x4 acc[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) acc[t] = f32x4{0, 0, 0, 0};
  for (int k0 = wave * 32; k0 < p.K; k0 += 128) {
    const int k = k0 + q * 8, kc = k < p.K ? k : 0;
    uint4 x = *reinterpret_cast<const uint4*>(hr + kc);
    if (k >= p.K) x = make_uint4(0, 0, 0, 0);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const uint4 v = *reinterpret_cast<const uint4*>(wr[t] + kc);
      acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, v), __builtin_bit_cast(bf16x8, x), acc[t], 0, 0, 0);
    }
  }
  // column r16: token; rows 4 q + r: experts
#pragma unroll
  for (int t = 0; t < NT; ++t) *reinterpret_cast<f32x4*>(&z_s[wave][r16][t * 16 + q * 4]) = acc[t];
  __syncthreads();
  for (int x = tid; x < 16 * NT * 16; x += 256) {
    const int t = x / (NT * 16), e = x % (NT * 16);
    z_s[0][t][e] = (z_s[0][t][e] + z_s[1][t][e]) + (z_s[2][t][e] + z_s[3][t][e]);
  }
  __syncthreads();
  const int64_t m = m0 + (tid >> 4);
  constexpr int NE = NT < 4 ? 4 : NT;
  choose<NE>(z_s[0][tid >> 4], p.Ex, p.top, tid & 15, [&](int j, int e, float z) {
    if ((tid & 15) == 0 && m < p.M) {
      p.ids[m * p.top + j] = e;
      p.scores[m * p.top + j] = sigmoid(z);
    }
  });
}

// ---------------------------------------------------------------------------------------------- prompts: sorting
// One workgroup per expert scans all A choices: how many belong to lower experts gives its first slot, a second pass
// writes its own.  rows[slot] = choice (token * top + j), slots[choice] = slot.  Expert e's tiles of TM slots are numbered
// from off / TM + e on, which leaves every expert room for its own; unused numbers are marked with expert -1.
constexpr int SORT_WAVES = 16;

__global__ __launch_bounds__(SORT_WAVES * 64) void moe_sort_kernel(const int* ids, int A, int Ex, int TM, int* rows, int* slots,
                                                                  int4* tiles, int n_tiles) {
  __shared__ int own_s[SORT_WAVES], low_s[SORT_WAVES];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, e = blockIdx.x;
  const int per = ((A + SORT_WAVES - 1) / SORT_WAVES + 63) / 64 * 64, i0 = wave * per, i1 = i0 + per < A ? i0 + per : A;
  int own = 0, low = 0;
#pragma unroll 4
  for (int i = i0 + lane; i < i1; i += 64) {
    const int id = ids[i];
    own += id == e;
    low += id < e;
  }
#pragma unroll
  for (int o = 32; o; o >>= 1) own += __shfl_xor(own, o, 64), low += __shfl_xor(low, o, 64);
  if (lane == 0) own_s[wave] = own, low_s[wave] = low;
  __syncthreads();
  int off = 0, cnt = 0, at = 0;
  for (int w = 0; w < SORT_WAVES; ++w) {
    off += low_s[w];
    at += w < wave ? own_s[w] : 0;
    cnt += own_s[w];
  }
  at += off;
  for (int ib = i0; ib < i1; ib += 64) {
    const int i = ib + lane;
    const bool mine = i < i1 && ids[i] == e;
    const uint64_t b = __builtin_amdgcn_ballot_w64(mine);
    if (mine) {
      const int s = at + __popcll(b & ((1ull << lane) - 1));
      rows[s] = i;
      slots[i] = s;
    }
    at += __popcll(b);
  }
  const int t0 = off / TM + e, mine = (cnt + TM - 1) / TM, t1 = e + 1 < Ex ? (off + cnt) / TM + e + 1 : n_tiles;
  for (int t = t0 + (int)threadIdx.x; t < t1 && t < n_tiles; t += SORT_WAVES * 64) {
    const int first = off + (t - t0) * TM, n = off + cnt - first;
    tiles[t] = t - t0 < mine ? make_int4(e, first, n < TM ? n : TM, 0) : make_int4(-1, 0, 0, 0);
  }
}

// ---------------------------------------------------------------------------------------------- prompts: grouped products
struct GroupArgs {
  const int4* tiles;    // (expert or -1, first slot, slots, -)
  const int* rows;      // slot -> choice
  const float* scores;  // by choice (GLU)
  int64_t ldx;
  int top, N, K;        // GLU: N = 2 F weight rows per expert, gate | up
};

// Any type and size: 64 slots x 64 weight rows (GLU: 32 gate and their 32 up rows), fp32 multiply-adds.
template <typename T, bool GLU>
__global__ __launch_bounds__(256) void grouped_any_kernel(GroupArgs p, const T* x, const T* w, T* out) {
  constexpr int TM = 64, BK = 16;
  __shared__ float x_s[BK][TM + 4], w_s[BK][64 + 4];
  __shared__ int64_t src_s[TM];
  __shared__ float sc_s[TM];
  const int4 tile = p.tiles[blockIdx.y];
  if (tile.x < 0) return;  // uniform
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4, F = GLU ? p.N / 2 : p.N;
  const int f0 = blockIdx.x * (GLU ? 32 : 64);
  if (tid < TM) {
    const int s = tile.y + (tid < tile.z ? tid : 0), c = p.rows[s];
    src_s[tid] = (int64_t)(GLU ? c / p.top : s) * p.ldx;
    sc_s[tid] = GLU ? p.scores[c] : 1.0f;
  }
  __syncthreads();
  const T* we = w + (int64_t)tile.x * p.N * p.K;
  float acc[4][4] = {};
  for (int k0 = 0; k0 < p.K; k0 += BK) {
    for (int i = tid; i < TM * BK; i += 256) {
      const int r = i / BK, k = i % BK;
      int n = f0 + (GLU ? r % 32 : r);
      const bool ok = n < F && k0 + k < p.K;
      if (GLU && r >= 32) n += F;
      x_s[k][r] = k0 + k < p.K ? to_f32(x[src_s[r] + k0 + k]) : 0.0f;
      w_s[k][r] = ok ? to_f32(we[(int64_t)n * p.K + k0 + k]) : 0.0f;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < BK; ++k) {
      float a[4], b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) a[i] = x_s[k][ty + 16 * i], b[i] = w_s[k][tx + 16 * i];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], b[j], acc[i][j]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = ty + 16 * i;
    if (r >= tile.z) continue;
#pragma unroll
    for (int j = 0; j < (GLU ? 2 : 4); ++j) {
      const int f = f0 + tx + 16 * j;
      if (f >= F) continue;
      const float v = GLU ? silu(sc_s[r] * acc[i][j]) * (sc_s[r] * acc[i][GLU ? j + 2 : j]) : acc[i][j];
      out[(int64_t)(tile.y + r) * F + f] = from_f32<T>(v);
    }
  }
}

// bf16 on the matrix cores.  Weights are the left operand (32 of them per accumulator's rows), slots the right one, so that a
// lane ends with four consecutive outputs of one slot.  A workgroup of 4 wavefronts, WM of them along the slots; a
// wavefront has 2 tiles of 32 weight rows (GLU: gate and up rows of the same outputs) and MT of 32 slots.
constexpr int GK = 64, GP = GK + 8;  // contraction per stage, row stride in LDS

template <int WM, int MT, bool GLU>
__global__ __launch_bounds__(256) void grouped_mfma_kernel(GroupArgs p, const uint16_t* x, const uint16_t* w, uint16_t* out) {
  constexpr int WN = 4 / WM, TM = WM * MT * 32, TN = WN * 64, XC = TM / 32, WC = TN / 32;
  extern __shared__ __align__(16) uint16_t lds[];  // 2 stages of TM + TN rows
  const int4 tile = p.tiles[blockIdx.y];
  if (tile.x < 0) return;  // uniform
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave % WM, wn = wave / WM;
  const int col = lane & 31, g2 = lane >> 5, F = GLU ? p.N / 2 : p.N, K = p.K;
  const int f0 = blockIdx.x * (GLU ? TN / 2 : TN);
  const int lr = tid >> 3, lc = (tid & 7) * 8;  // this thread's row (of every 32) and column in a stage
  const uint16_t* xp[XC];
  const uint16_t* wp[WC];
#pragma unroll
  for (int i = 0; i < XC; ++i) {
    const int r = i * 32 + lr, s = tile.y + (r < tile.z ? r : 0);
    xp[i] = x + (int64_t)(GLU ? p.rows[s] / p.top : s) * p.ldx + lc;
  }
  const uint16_t* we = w + (int64_t)tile.x * p.N * K + lc;
#pragma unroll
  for (int i = 0; i < WC; ++i) {
    // GLU: rows of 64 alternate 32 gate and 32 up rows, a wavefront's two tiles
    int n = f0 + (GLU ? i / 2 * 32 : i * 32) + lr;
    n = n < F ? n : F - 1;
    wp[i] = we + (int64_t)(GLU && (i & 1) ? n + F : n) * K;
  }
  uint4 xr[XC], wr[WC];
  auto fetch = [&](int k0) __attribute__((always_inline)) {
    const bool ok = k0 + lc < K;
    const int k = ok ? k0 : 0;
#pragma unroll
    for (int i = 0; i < XC; ++i) {
      xr[i] = *reinterpret_cast<const uint4*>(xp[i] + (ok ? k : -lc));
      if (!ok) xr[i] = make_uint4(0, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < WC; ++i) wr[i] = *reinterpret_cast<const uint4*>(wp[i] + (ok ? k : -lc));
  };
  auto stage = [&](int buf) __attribute__((always_inline)) {
    uint16_t* xs = lds + buf * (TM + TN) * GP;
    uint16_t* ws = xs + TM * GP;
#pragma unroll
    for (int i = 0; i < XC; ++i) *reinterpret_cast<uint4*>(&xs[(i * 32 + lr) * GP + lc]) = xr[i];
#pragma unroll
    for (int i = 0; i < WC; ++i) *reinterpret_cast<uint4*>(&ws[(i * 32 + lr) * GP + lc]) = wr[i];
  };
  f32x16 acc[2][MT];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < MT; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.0f;
  fetch(0);
  stage(0);
  __syncthreads();
  int buf = 0;
  for (int k0 = 0; k0 < K; k0 += GK, buf ^= 1) {
    const bool more = k0 + GK < K;
    if (more) fetch(k0 + GK);
    const uint16_t* xs = lds + buf * (TM + TN) * GP + (wm * MT * 32 + col) * GP + g2 * 8;
    const uint16_t* ws = lds + buf * (TM + TN) * GP + (TM + wn * 64 + col) * GP + g2 * 8;
#pragma unroll
    for (int kk = 0; kk < GK / 16; ++kk) {
      bf16x8 a[2], b[MT];
#pragma unroll
      for (int i = 0; i < 2; ++i) a[i] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(ws + i * 32 * GP + kk * 16));
#pragma unroll
      for (int j = 0; j < MT; ++j) b[j] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(xs + j * 32 * GP + kk * 16));
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < MT; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[i], b[j], acc[i][j], 0, 0, 0);
    }
    if (more) stage(buf ^ 1);
    __syncthreads();
  }
  // register r of a tile: weight row 8 (r / 4) + 4 g2 + r % 4, slot col
#pragma unroll
  for (int j = 0; j < MT; ++j) {
    const int r = wm * MT * 32 + j * 32 + col;
    if (r >= tile.z) continue;
    uint16_t* dst = out + (int64_t)(tile.y + r) * F;
    if constexpr (GLU) {
      const float sc = p.scores[p.rows[tile.y + r]];
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int f = f0 + wn * 32 + 8 * q + 4 * g2;
        if (f >= F) continue;
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = silu(sc * acc[0][j][4 * q + e]) * (sc * acc[1][j][4 * q + e]);
        *reinterpret_cast<uint2*>(dst + f) = make_uint2(pack2(v[0], v[1]), pack2(v[2], v[3]));
      }
    } else {
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int q = 0; q < 4; ++q) {
          const int f = f0 + wn * 64 + i * 32 + 8 * q + 4 * g2;
          if (f >= F) continue;
          *reinterpret_cast<uint2*>(dst + f) = make_uint2(pack2(acc[i][j][4 * q], acc[i][j][4 * q + 1]), pack2(acc[i][j][4 * q + 2], acc[i][j][4 * q + 3]));
        }
    }
  }
}

// ---------------------------------------------------------------------------------------------- steps of a few tokens
// Dot products of R rows of w (row i at w[i]) with x over K elements by one wavefront; K a multiple of 8
template <typename T, int R>
__device__ __forceinline__ void dot_rows(const T* const (&w)[R], const T* x, int K, int lane, float (&acc)[R]) {
  constexpr int U = R <= 2 ? 4 : 2;
  for (int k0 = lane * 8; k0 < K; k0 += 512 * U) {
    Raw8<T> wv[R][U], xv[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * 512 < K ? k0 + u * 512 : 0;
      xv[u].load(x + k);
#pragma unroll
      for (int i = 0; i < R; ++i) wv[i][u].load(w[i] + k);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      float f[8], g[8];
      xv[u].get(f);
      const bool on = k0 + u * 512 < K;
#pragma unroll
      for (int i = 0; i < R; ++i) {
        wv[i][u].get(g);
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[i] = fmaf(g[e], on ? f[e] : 0.0f, acc[i]);
      }
    }
  }
}

// h [M, K], z [M, Ex] router logits -> act [M * top, F] of the chosen experts (w [Ex, 2 F, K])
template <typename T>
__global__ __launch_bounds__(256) void moe_up_kernel(const T* h, const float* z, const T* w, T* act, int K, int F, int Ex, int top) {
  constexpr int OR = 2;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = blockIdx.y, m = blockIdx.z;
  const int f0 = (blockIdx.x * 4 + wave) * OR;
  int expert = 0;
  float score = 0.0f;
  choose_any(z + (int64_t)m * Ex, Ex, j + 1, lane & 15, [&](int, int e, float v) { expert = e, score = v; });
  expert = __builtin_amdgcn_readfirstlane(expert);
  if (f0 >= F) return;
  const T* wr[2 * OR];
#pragma unroll
  for (int i = 0; i < 2 * OR; ++i) {
    const int f = f0 + i % OR < F ? f0 + i % OR : F - 1;
    wr[i] = w + ((int64_t)expert * 2 * F + (i < OR ? f : f + F)) * K;
  }
  float acc[2 * OR] = {};
  dot_rows<T, 2 * OR>(wr, h + (int64_t)m * K, K, lane, acc);
  const float s = sigmoid(score);
#pragma unroll
  for (int i = 0; i < OR; ++i) {
    const float g = s * wave_sum(acc[i]), u = s * wave_sum(acc[i + OR]);
    if (lane == 0 && f0 + i < F) act[((int64_t)m * top + j) * F + f0 + i] = from_f32<T>(silu(g) * u);
  }
}

// y [M, N] = sum over the chosen experts of W_down act, plus the shared expert's (sw [N, Fs], sact [M, Fs]; Fs 0: none)
template <typename T>
__global__ __launch_bounds__(256) void moe_down_kernel(const float* z, const T* act, const T* w, const T* sact, const T* sw, float* y,
                                                       int N, int F, int Fs, int Ex, int top) {
  constexpr int R = 2;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, m = blockIdx.y;
  const int n0 = (blockIdx.x * 4 + wave) * R;
  if (n0 >= N) return;
  float acc[R] = {};
  const T* wr[R];
  auto rows = [&](const T* base, int K) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < R; ++i) wr[i] = base + (int64_t)(n0 + i < N ? n0 + i : N - 1) * K;
  };
  if (Fs) {
    rows(sw, Fs);
    dot_rows<T, R>(wr, sact + (int64_t)m * Fs, Fs, lane, acc);
  }
  choose_any(z + (int64_t)m * Ex, Ex, top, lane & 15, [&](int j, int e, float) {
    rows(w + (int64_t)__builtin_amdgcn_readfirstlane(e) * N * F, F);
    dot_rows<T, R>(wr, act + ((int64_t)m * top + j) * F, F, lane, acc);
  });
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const float s = wave_sum(acc[i]);
    if (lane == 0 && n0 + i < N) y[(int64_t)m * N + n0 + i] = s;
  }
}

// the matrix-core product for these operands
inline bool mfma_ok(int dtype, int64_t ldx, int64_t N, int64_t K, bool glu, const void* x, const void* w, const void* out) {
  return dtype == AQ_BF16 && K % 8 == 0 && ldx % 8 == 0 && (glu ? N / 2 : N) % 4 == 0 && !bad_ptr16(x) && !bad_ptr16(w) && !bad_ptr16(out);
}

}  // namespace sq

using namespace sq;

extern "C" int aqs_moe_route(const void* h, int64_t ldh, int dtype, const void* w, int32_t* ids, float* scores, int64_t M, int64_t K,
                             int64_t Ex, int64_t top, void* stream) {
  SQ_CHECK(M >= 0 && K > 0 && Ex > 0 && top > 0 && top <= Ex && ldh >= K, AQ_E_SHAPE);
  SQ_CHECK(Ex <= MAX_EXPERTS && M < (1 << 24) && M * top < ((int64_t)1 << 31) && K < (1 << 24), AQ_E_RANGE);
  if (M == 0) return AQ_OK;
  SQ_NEED(h && w && ids && scores);
  const RouteArgs p{ids, scores, ldh, (int)M, (int)K, (int)Ex, (int)top};
  hipStream_t st = (hipStream_t)stream;
  if (dtype == AQ_BF16 && K % 8 == 0 && ldh % 8 == 0 && !bad_ptr16(h) && !bad_ptr16(w) && Ex <= 224) {
    const unsigned grid = (unsigned)((M + 15) / 16);
    const uint16_t *hp = (const uint16_t*)h, *wp = (const uint16_t*)w;
    if (Ex <= 32) route_mfma_kernel<2><<<grid, 256, 0, st>>>(p, hp, wp);
    else if (Ex <= 64) route_mfma_kernel<4><<<grid, 256, 0, st>>>(p, hp, wp);
    else if (Ex <= 128) route_mfma_kernel<8><<<grid, 256, 0, st>>>(p, hp, wp);
    else route_mfma_kernel<14><<<grid, 256, 0, st>>>(p, hp, wp);
    return launched();
  }
  SQ_DISPATCH(dtype, (route_any_kernel<T><<<dim3((unsigned)((M + 3) / 4)), 256, 0, st>>>(p, (const T*)h, (const T*)w)));
  return launched();
}

// slots per tile for A choices of Ex experts of width K and inner size F
extern "C" int64_t aqs_moe_tile(int dtype, int64_t A, int64_t Ex, int64_t K, int64_t F) {
  if (dtype != AQ_BF16 || K % 8 || F % 8) return 64;
  return A >= 64 * Ex ? 128 : 32;
}
extern "C" int64_t aqs_moe_tiles(int64_t A, int64_t Ex, int64_t tile) { return A / tile + Ex + 1; }

extern "C" int aqs_moe_sort(const int32_t* ids, int64_t A, int64_t Ex, int64_t tile, int32_t* rows, int32_t* slots, int32_t* tiles,
                            int64_t n_tiles, void* stream) {
  SQ_CHECK(A >= 0 && Ex > 0 && tile > 0 && n_tiles == aqs_moe_tiles(A, Ex, tile), AQ_E_SHAPE);
  SQ_CHECK(Ex <= MAX_EXPERTS && A < (1 << 30), AQ_E_RANGE);
  if (A == 0) return AQ_OK;
  SQ_NEED(ids && rows && slots && tiles);
  SQ_CHECK(!bad_ptr16(tiles), AQ_E_ALIGN);
  moe_sort_kernel<<<dim3((unsigned)Ex), SORT_WAVES * 64, 0, (hipStream_t)stream>>>(ids, (int)A, (int)Ex, (int)tile, rows, slots,
                                                                                  (int4*)tiles, (int)n_tiles);
  return launched();
}

// glu != 0: x [tokens, ldx], w [Ex, N = 2 F, K] gate | up, out [A, F] = silu(s g) (s u); otherwise x [A, ldx] by slot, out [A, N].
extern "C" int aqs_moe_product(int glu, const void* x, int64_t ldx, int dtype, const void* w, const int32_t* tiles, int64_t n_tiles,
                               int64_t tile, const int32_t* rows, const float* scores, int64_t top, void* out, int64_t N, int64_t K,
                               void* stream) {
  SQ_CHECK(N > 0 && K > 0 && top > 0 && n_tiles > 0 && ldx >= K && (!glu || N % 2 == 0), AQ_E_SHAPE);
  SQ_CHECK(n_tiles < 65536 && N < (1 << 24) && K < (1 << 24), AQ_E_RANGE);
  SQ_NEED(x && w && tiles && rows && out && (scores || !glu));
  const GroupArgs p{(const int4*)tiles, rows, scores, ldx, (int)top, (int)N, (int)K};
  const int64_t F = glu ? N / 2 : N;
  hipStream_t st = (hipStream_t)stream;
  if (tile == 64) {
    const dim3 grid((unsigned)((F + (glu ? 31 : 63)) / (glu ? 32 : 64)), (unsigned)n_tiles);
    SQ_DISPATCH(dtype, if (glu)(grouped_any_kernel<T, true><<<grid, 256, 0, st>>>(p, (const T*)x, (const T*)w, (T*)out));
                else (grouped_any_kernel<T, false><<<grid, 256, 0, st>>>(p, (const T*)x, (const T*)w, (T*)out)));
    return launched();
  }
  SQ_CHECK(mfma_ok(dtype, ldx, N, K, glu, x, w, out), AQ_E_ALIGN);
  auto go = [&](auto wm_tag, auto mt_tag, auto glu_tag) -> int {
    constexpr int WM = decltype(wm_tag)::value, MT = decltype(mt_tag)::value, TM = WM * MT * 32, TN = 4 / WM * 64;
    constexpr bool G = decltype(glu_tag)::value;
    auto* k = grouped_mfma_kernel<WM, MT, G>;
    constexpr size_t lds = (size_t)2 * (TM + TN) * GP * 2;
    if (lds > 64 * 1024) {
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    constexpr int cols = G ? TN / 2 : TN;
    k<<<dim3((unsigned)((F + cols - 1) / cols), (unsigned)n_tiles), 256, lds, st>>>(p, (const uint16_t*)x, (const uint16_t*)w, (uint16_t*)out);
    return launched();
  };
  using std::integral_constant;
  if (tile == 128) {
    if (glu) return go(integral_constant<int, 2>{}, integral_constant<int, 2>{}, std::true_type{});
    return go(integral_constant<int, 2>{}, integral_constant<int, 2>{}, std::false_type{});
  }
  SQ_CHECK(tile == 32, AQ_E_SHAPE);
  if (glu) return go(integral_constant<int, 1>{}, integral_constant<int, 1>{}, std::true_type{});
  return go(integral_constant<int, 1>{}, integral_constant<int, 1>{}, std::false_type{});
}

// whether the two launches below serve these sizes
extern "C" int aqs_moe_step_ok(int64_t M, int64_t N, int64_t F, int64_t Fs, int64_t Ex, int64_t top) {
  return M > 0 && M <= 8 && N > 0 && N % 8 == 0 && F > 0 && F % 8 == 0 && Fs >= 0 && Fs % 8 == 0 && Ex > 0 && Ex <= MAX_EXPERTS && top > 0 &&
         top <= Ex;
}

// h [M, K], z [M, Ex] logits, w [Ex, 2 F, K] -> act [M * top, F]
extern "C" int aqs_moe_step_up(const void* h, const float* z, int dtype, const void* w, void* act, int64_t M, int64_t K, int64_t F,
                               int64_t Ex, int64_t top, void* stream) {
  SQ_CHECK(aqs_moe_step_ok(M, K, F, 0, Ex, top), AQ_E_SHAPE);
  SQ_NEED(h && z && w && act);
  SQ_CHECK(!bad_ptr16(h) && !bad_ptr16(w), AQ_E_ALIGN);
  const dim3 grid((unsigned)((F + 7) / 8), (unsigned)top, (unsigned)M);
  SQ_DISPATCH(dtype, (moe_up_kernel<T><<<grid, 256, 0, (hipStream_t)stream>>>((const T*)h, z, (const T*)w, (T*)act, (int)K, (int)F, (int)Ex, (int)top)));
  return launched();
}

// act [M * top, F], w [Ex, N, F], shared sact [M, Fs] and sw [N, Fs] (Fs 0: none) -> y [M, N] fp32
extern "C" int aqs_moe_step_down(const float* z, const void* act, int dtype, const void* w, const void* sact, const void* sw, float* y,
                                 int64_t M, int64_t N, int64_t F, int64_t Fs, int64_t Ex, int64_t top, void* stream) {
  SQ_CHECK(aqs_moe_step_ok(M, N, F, Fs, Ex, top), AQ_E_SHAPE);
  SQ_NEED(z && act && w && y && (Fs == 0 || (sact && sw)));
  SQ_CHECK(!bad_ptr16(act) && !bad_ptr16(w) && !bad_ptr16(sact) && !bad_ptr16(sw), AQ_E_ALIGN);
  const dim3 grid((unsigned)((N + 7) / 8), (unsigned)M);
  SQ_DISPATCH(dtype, (moe_down_kernel<T><<<grid, 256, 0, (hipStream_t)stream>>>(z, (const T*)act, (const T*)w, (const T*)sact, (const T*)sw, y,
                                                                                (int)N, (int)F, (int)Fs, (int)Ex, (int)top)));
  return launched();
}
