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

// bf16 on the matrix cores: 16 tokens per workgroup, every wavefront all experts over its share of the contraction.  NT:
// tiles of 16 experts; KU: products whose operands are requested together (in pairs that read whole cache lines
// of a row); NW: wavefronts.
template <int NT, int KU, int NW>
__global__ __launch_bounds__(NW * 64) void route_mfma_kernel(RouteArgs p, const uint16_t* h, const uint16_t* w) {
  constexpr int ZP = NT * 16 + 4;
  __shared__ __align__(16) float z_s[NW][16][ZP];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, q = lane >> 4;
  const int64_t m0 = (int64_t)blockIdx.x * 16;
  const uint16_t* hr = h + (m0 + r16 < p.M ? m0 + r16 : p.M - 1) * p.ldh;
  const uint16_t* wr[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) wr[t] = w + (int64_t)(t * 16 + r16 < p.Ex ? t * 16 + r16 : p.Ex - 1) * p.K;
  f32x4 acc[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) acc[t] = f32x4{0, 0, 0, 0};
  static_assert(KU % 2 == 0, "whole cache lines");
  for (int k0 = wave * 64; k0 < p.K; k0 += NW * 32 * KU) {
    uint4 x[KU], v[KU][NT];
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      const int k = k0 + u / 2 * NW * 64 + (q * 2 + u % 2) * 8, kc = k < p.K ? k : 0;
      x[u] = *reinterpret_cast<const uint4*>(hr + kc);
#pragma unroll
      for (int t = 0; t < NT; ++t) v[u][t] = *reinterpret_cast<const uint4*>(wr[t] + kc);
    }
    __builtin_amdgcn_sched_barrier(0);  // all of them are requested before the first is waited for
#pragma unroll
    for (int u = 0; u < KU; ++u) {
      if (k0 + u / 2 * NW * 64 + (q * 2 + u % 2) * 8 >= p.K) x[u] = make_uint4(0, 0, 0, 0);
#pragma unroll
      for (int t = 0; t < NT; ++t)
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, v[u][t]), __builtin_bit_cast(bf16x8, x[u]), acc[t], 0, 0, 0);
    }
  }
  // column r16: token; rows 4 q + r: experts
#pragma unroll
  for (int t = 0; t < NT; ++t) *reinterpret_cast<f32x4*>(&z_s[wave][r16][t * 16 + q * 4]) = acc[t];
  __syncthreads();
  for (int x = tid; x < 16 * NT * 16; x += NW * 64) {
    const int t = x / (NT * 16), e = x % (NT * 16);
    float v = z_s[0][t][e];
#pragma unroll
    for (int i = 1; i < NW; ++i) v += z_s[i][t][e];
    z_s[0][t][e] = v;
  }
  __syncthreads();
  if (tid >= 256) return;
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
// One workgroup per expert counts all A choices by expert, which gives its first slot and its first tile; a second pass
// writes its own: rows[slot] = choice (token * top + j), slots[choice] = slot.  tiles[0].x = number of tiles, tiles[1 ..] =
// (expert, first slot, slots of the tile, -).
constexpr int SORT_WAVES = 16;

__global__ __launch_bounds__(SORT_WAVES * 64) void moe_sort_kernel(const int* ids, int A, int Ex, int TM, int* rows, int* slots,
                                                                  int4* tiles, int n_tiles) {
  __shared__ int own_s[SORT_WAVES], count_s[MAX_EXPERTS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, e = blockIdx.x;
  for (int i = tid; i < Ex; i += SORT_WAVES * 64) count_s[i] = 0;
  __syncthreads();
  const int per = ((A + SORT_WAVES - 1) / SORT_WAVES + 63) / 64 * 64, i0 = wave * per, i1 = i0 + per < A ? i0 + per : A;
  int own = 0;
  constexpr int U = 8;  // reads together
  for (int ib = i0; ib < i1; ib += 64 * U) {
    int id[U];
#pragma unroll
    for (int u = 0; u < U; ++u) id[u] = ids[ib + u * 64 + lane < i1 ? ib + u * 64 + lane : i0];
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (ib + u * 64 + lane < i1) {
        own += id[u] == e;
        atomicAdd(&count_s[id[u]], 1);
      }
  }
#pragma unroll
  for (int o = 32; o; o >>= 1) own += __shfl_xor(own, o, 64);
  if (lane == 0) own_s[wave] = own;
  __syncthreads();
  int off = 0, t0 = 0, total = 0;  // every wavefront sums for itself
  for (int i = lane; i < Ex; i += 64) {
    const int c = count_s[i], t = (c + TM - 1) / TM;
    off += i < e ? c : 0;
    t0 += i < e ? t : 0;
    total += t;
  }
#pragma unroll
  for (int o = 32; o; o >>= 1) off += __shfl_xor(off, o, 64), t0 += __shfl_xor(t0, o, 64), total += __shfl_xor(total, o, 64);
  const int cnt = count_s[e];
  int at = off;
  for (int w = 0; w < wave; ++w) at += own_s[w];
  for (int ib = i0; ib < i1; ib += 64 * U) {
    int id[U];
#pragma unroll
    for (int u = 0; u < U; ++u) id[u] = ids[ib + u * 64 + lane < i1 ? ib + u * 64 + lane : i0];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int i = ib + u * 64 + lane;
      const bool mine = i < i1 && id[u] == e;
      const uint64_t b = __builtin_amdgcn_ballot_w64(mine);
      if (mine) {
        const int s = at + __popcll(b & ((1ull << lane) - 1));
        rows[s] = i;
        slots[i] = s;
      }
      at += __popcll(b);
    }
  }
  if (e == 0 && tid == 0) tiles[0] = make_int4(total, 0, 0, 0);
  for (int t = tid; t * TM < cnt && 1 + t0 + t < n_tiles; t += SORT_WAVES * 64)
    tiles[1 + t0 + t] = make_int4(e, off + t * TM, cnt - t * TM < TM ? cnt - t * TM : TM, 0);
}

// ---------------------------------------------------------------------------------------------- prompts: grouped products
struct GroupArgs {
  const int4* tiles;    // [0].x: how many; [1 ..]: (expert, first slot, slots, -)
  const int* rows;      // slot -> choice
  const float* scores;  // by choice (GLU)
  int64_t ldx, x_bytes; // x_bytes: extent of x's rows (matrix cores)
  int top, N, K;        // GLU: N = 2 F weight rows per expert, gate | up
};

// Any type and size: 64 slots x 64 weight rows (GLU: 32 gate and their 32 up rows), fp32 multiply-adds.
template <typename T, bool GLU>
__global__ __launch_bounds__(256) void grouped_any_kernel(GroupArgs p, const T* x, const T* w, T* out) {
  constexpr int TM = 64, BK = 16;
  __shared__ float x_s[BK][TM + 4], w_s[BK][64 + 4];
  __shared__ int64_t src_s[TM];
  __shared__ float sc_s[TM];
  if ((int)blockIdx.y >= p.tiles[0].x) return;  // uniform
  const int4 tile = p.tiles[1 + blockIdx.y];
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
// lane ends with four consecutive outputs of one slot.  WW x WT wavefronts, each with 2 tiles of 32 weight rows (GLU: the
// gate and the up rows of the same 32 outputs) and JT of 32 slots.  The contraction is walked in steps of 64 through NS
// stages in LDS, filled by direct global->LDS loads: a load brings 8 rows of 128 bytes, whose 16-byte pieces are permuted
// (piece c of row r in place c ^ (r / 2) % 8) so that 16 rows' reads of one piece meet no bank twice.
template <int WW_, int WT_, int JT_, int NS_>
struct GroupShape {
  static constexpr int WW = WW_, WT = WT_, JT = JT_, NS = NS_, NW = WW * WT, THREADS = NW * 64;
  static constexpr int WROWS = WW * 64, TROWS = WT * JT * 32, STAGE = (WROWS + TROWS) * 128;
  static constexpr int W_LOADS = WROWS / 8 / NW, T_LOADS = TROWS / 8 / NW, LOADS = W_LOADS + T_LOADS;
  static_assert(NW % 2 == 0, "a wavefront's rows of all its loads are permuted alike");
  static_assert(TROWS % (8 * NW) == 0 && NS * STAGE <= 160 * 1024 && (NS - 1) * LOADS < 64, "whole loads, LDS, counter");
};
using GroupWide = GroupShape<4, 2, 2, 3>;    // 256 weight rows x 128 slots
using GroupNarrow = GroupShape<2, 1, 1, 4>;  // 128 weight rows x 32 slots: weights stream by

typedef __attribute__((address_space(3))) void lds_void;
// until at most n vector loads are on their way, and no LDS read
#define SQ_WAIT_VM_LDS(n) __builtin_amdgcn_s_waitcnt(0x0070 | ((n) & 15) | (((n) >> 4) << 14))
// a workgroup barrier without the fence of __syncthreads(), which would wait for the loads of later stages
#define SQ_RAW_BARRIER()           \
  do {                             \
    asm volatile("" ::: "memory"); \
    __builtin_amdgcn_s_barrier();  \
    asm volatile("" ::: "memory"); \
  } while (0)
constexpr uint32_t GROUP_OOB = 0x7ffffff0u;  // beyond every descriptor: reads zero

template <class G, bool GLU>
__device__ __forceinline__ void grouped_tile(const GroupArgs& p, const uint16_t* x, const uint16_t* w, uint16_t* out, uint8_t* smem) {
  // consecutive workgroups go to different XCDs: number them so that each XCD takes a run of tiles, outputs first
  const int cols = (int)gridDim.x, total = cols * p.tiles[0].x, pid = blockIdx.y * cols + blockIdx.x;
  if (pid >= total) return;  // uniform
  const int per = total / 8, rem = total % 8, xcd = pid % 8, id = xcd * per + (xcd < rem ? xcd : rem) + pid / 8;
  const int4 tile = p.tiles[1 + id / cols];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), ww = wave % G::WW, wt = wave / G::WW;
  const int col = lane & 31, g2 = lane >> 5, F = GLU ? p.N / 2 : p.N, K = p.K;
  const int f0 = id % cols * (GLU ? G::WROWS / 2 : G::WROWS);
  const __amdgpu_buffer_rsrc_t Wr =
      __builtin_amdgcn_make_buffer_rsrc(const_cast<uint16_t*>(w + (int64_t)tile.x * p.N * K), 0, (int)((int64_t)p.N * K * 2), 0x00020000);
  const __amdgpu_buffer_rsrc_t Xr = __builtin_amdgcn_make_buffer_rsrc(const_cast<uint16_t*>(x), 0, (int)p.x_bytes, 0x00020000);
  // this lane's row of every load, and its piece of it
  const int lr = wave * 8 + lane / 8, piece = ((lane % 8) ^ (lr / 2 % 8)) * 16;
  uint32_t wo[G::W_LOADS], xo[G::T_LOADS];
#pragma unroll
  for (int i = 0; i < G::W_LOADS; ++i) {
    const int r = i * 8 * G::NW + lr, n = f0 + (GLU ? r / 64 * 32 + r % 32 : r);
    wo[i] = n < F ? (uint32_t)(GLU && (r & 32) ? n + F : n) * (uint32_t)K * 2 + piece : GROUP_OOB;
  }
#pragma unroll
  for (int i = 0; i < G::T_LOADS; ++i) {
    const int r = i * 8 * G::NW + lr, s = tile.y + (r < tile.z ? r : 0);
    xo[i] = r < tile.z ? (uint32_t)(GLU ? p.rows[s] / p.top : s) * (uint32_t)(p.ldx * 2) + piece : GROUP_OOB;
  }
  const int nk = (K + 63) / 64;
  auto fetch = [&](int kt) __attribute__((always_inline)) {
    uint8_t* st = smem + kt % G::NS * G::STAGE + wave * 1024;
    const uint32_t k0 = (uint32_t)kt * 128;
    const bool ok = (int)k0 + piece < K * 2;  // past the end, zeros: the number of loads in flight stays the same
#pragma unroll
    for (int i = 0; i < G::W_LOADS; ++i)
      __builtin_amdgcn_raw_ptr_buffer_load_lds(Wr, (lds_void*)(st + i * 1024 * G::NW), 16, ok ? wo[i] + k0 : GROUP_OOB, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < G::T_LOADS; ++i)
      __builtin_amdgcn_raw_ptr_buffer_load_lds(Xr, (lds_void*)(st + G::WROWS * 128 + i * 1024 * G::NW), 16, ok ? xo[i] + k0 : GROUP_OOB, 0, 0, 0);
  };
  f32x16 acc[2][G::JT];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < G::JT; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.0f;
  // Fragments are read a quarter of a stage ahead of their products.  When the last quarter's are in registers (and the
  // next stage has landed), a barrier frees the stage for the loads of the one NS later.
  const int fw = (ww * 64 + col) * 128, fx = (G::WROWS + wt * G::JT * 32 + col) * 128, turn = col / 2 % 8;
  bf16x8 a[2][2], b[2][G::JT];
  auto read = [&](int s, int kk, int f, int to) __attribute__((always_inline)) {  // fragment f: 0, 1 of the weights, then slots
    const uint8_t* st = smem + s % G::NS * G::STAGE + ((kk * 2 + g2) ^ turn) * 16;
    if (f < 2) a[to][f] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(st + fw + f * 32 * 128));
    else b[to][f - 2] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(st + fx + (f - 2) * 32 * 128));
  };
#pragma unroll
  for (int s = 0; s < G::NS; ++s) fetch(s);
  SQ_WAIT_VM_LDS((G::NS - 1) * G::LOADS);
  SQ_RAW_BARRIER();
  // JN: the wavefront's tiles that hold slots at all
  auto run = [&](auto tag) __attribute__((always_inline)) {
    constexpr int JN = decltype(tag)::value, NF = JN ? 2 + JN : 0, NM = JN ? 2 * JN : 1;
    auto quarter = [&](int from, int s, int kk) __attribute__((always_inline)) {  // products; the fragments of (s, kk) read beside
#pragma unroll
      for (int m = 0; m < 2 * JN; ++m) {
        acc[m % 2][m / 2] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[from][m % 2], b[from][m / 2], acc[m % 2][m / 2], 0, 0, 0);
#pragma unroll
        for (int f = m * NF / NM; f < (m + 1) * NF / NM; ++f) read(s, kk, f, from ^ 1);
        __builtin_amdgcn_sched_barrier(0);
      }
    };
#pragma unroll
    for (int f = 0; f < NF; ++f) read(0, 0, f, 0);
    for (int s = 0; s < nk; ++s) {
      quarter(0, s, 1);
      quarter(1, s, 2);
      quarter(0, s, 3);
      SQ_WAIT_VM_LDS((G::NS - 2) * G::LOADS);
      SQ_RAW_BARRIER();
      fetch(s + G::NS);
      quarter(1, s + 1, 0);
    }
  };
  const int held = tile.z - wt * G::JT * 32;
  if (held <= 0) run(std::integral_constant<int, 0>{});
  else if (G::JT > 1 && held <= 32) run(std::integral_constant<int, 1>{});
  else run(std::integral_constant<int, G::JT>{});
  SQ_WAIT_VM_LDS(0);  // the padding loads, before the workgroup's LDS goes to another
  // register r of a tile: weight row 8 (r / 4) + 4 g2 + r % 4, slot col
#pragma unroll
  for (int j = 0; j < G::JT; ++j) {
    const int r = (wt * G::JT + j) * 32 + col;
    if (r >= tile.z) continue;
    uint16_t* dst = out + (int64_t)(tile.y + r) * F;
    if constexpr (GLU) {
      const float sc = p.scores[p.rows[tile.y + r]];
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int f = f0 + ww * 32 + 8 * q + 4 * g2;
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
          const int f = f0 + ww * 64 + i * 32 + 8 * q + 4 * g2;
          if (f >= F) continue;
          *reinterpret_cast<uint2*>(dst + f) = make_uint2(pack2(acc[i][j][4 * q], acc[i][j][4 * q + 1]), pack2(acc[i][j][4 * q + 2], acc[i][j][4 * q + 3]));
        }
    }
  }
}

template <class G, bool GLU>
__global__ __launch_bounds__(G::THREADS) void grouped_mfma_kernel(GroupArgs p, const uint16_t* x, const uint16_t* w, uint16_t* out) {
  __shared__ __attribute__((aligned(1024))) uint8_t smem[G::NS * G::STAGE];
  grouped_tile<G, GLU>(p, x, w, out, smem);
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
  int mine = 0;  // lane j: expert j
  choose_any(z + (int64_t)m * Ex, Ex, top, lane & 15, [&](int j, int e, float) { mine = lane == j ? e : mine; });
  // the experts' rows as one sequence of pieces of 512, four pieces together
  constexpr int U = 4;
  const int steps = (F + 511) / 512, total = top * steps;
  int j = 0, st = 0;
  for (int s0 = 0; s0 < total; s0 += U) {
    Raw8<T> wv[R][U], xv[U];
    bool on[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int f = st * 512 + lane * 8, fc = f < F ? f : 0;
      on[u] = f < F && s0 + u < total;
      xv[u].load(act + ((int64_t)m * top + j) * F + fc);
      rows(w + (int64_t)__builtin_amdgcn_readlane(mine, j) * N * F, F);
#pragma unroll
      for (int i = 0; i < R; ++i) wv[i][u].load(wr[i] + fc);
      if (++st == steps) st = 0, j = j + 1 < top ? j + 1 : j;
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      float f[8], g[8];
      xv[u].get(f);
#pragma unroll
      for (int i = 0; i < R; ++i) {
        wv[i][u].get(g);
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[i] = fmaf(g[e], on[u] ? f[e] : 0.0f, acc[i]);
      }
    }
  }
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
    if (Ex <= 32) route_mfma_kernel<2, 8, 8><<<grid, 512, 0, st>>>(p, hp, wp);
    else if (Ex <= 64) route_mfma_kernel<4, 8, 8><<<grid, 512, 0, st>>>(p, hp, wp);
    else if (Ex <= 96) route_mfma_kernel<6, 4, 8><<<grid, 512, 0, st>>>(p, hp, wp);
    else if (Ex <= 128) route_mfma_kernel<8, 6, 4><<<grid, 256, 0, st>>>(p, hp, wp);
    else route_mfma_kernel<14, 2, 4><<<grid, 256, 0, st>>>(p, hp, wp);
    return launched();
  }
  SQ_DISPATCH(dtype, (route_any_kernel<T><<<dim3((unsigned)((M + 3) / 4)), 256, 0, st>>>(p, (const T*)h, (const T*)w)));
  return launched();
}

// slots per tile for A choices of Ex experts of width K and inner size F
extern "C" int64_t aqs_moe_tile(int dtype, int64_t A, int64_t Ex, int64_t K, int64_t F) {
  if (dtype != AQ_BF16 || K % 8 || F % 8) return 64;
  return A >= 64 * Ex ? GroupWide::TROWS : GroupNarrow::TROWS;
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
                               int64_t tile, const int32_t* rows, const float* scores, int64_t A, int64_t top, void* out, int64_t N,
                               int64_t K, void* stream) {
  SQ_CHECK(N > 0 && K > 0 && A > 0 && top > 0 && A % top == 0 && n_tiles > 1 && ldx >= K && (!glu || N % 2 == 0), AQ_E_SHAPE);
  SQ_CHECK(n_tiles < 65536 && N < (1 << 24) && K < (1 << 24), AQ_E_RANGE);
  SQ_NEED(x && w && tiles && rows && out && (scores || !glu));
  // extent of x's rows: whole rows but for the last one's padding
  const int64_t x_rows = glu ? A / top : A, x_bytes = ((x_rows - 1) * ldx + K) * 2;
  const GroupArgs p{(const int4*)tiles, rows, scores, ldx, x_bytes, (int)top, (int)N, (int)K};
  const int64_t F = glu ? N / 2 : N;
  hipStream_t st = (hipStream_t)stream;
  if (tile == 64) {
    const dim3 grid((unsigned)((F + (glu ? 31 : 63)) / (glu ? 32 : 64)), (unsigned)(n_tiles - 1));
    SQ_DISPATCH(dtype, if (glu)(grouped_any_kernel<T, true><<<grid, 256, 0, st>>>(p, (const T*)x, (const T*)w, (T*)out));
                else (grouped_any_kernel<T, false><<<grid, 256, 0, st>>>(p, (const T*)x, (const T*)w, (T*)out)));
    return launched();
  }
  SQ_CHECK(mfma_ok(dtype, ldx, N, K, glu, x, w, out), AQ_E_ALIGN);
  SQ_CHECK(x_bytes < (int64_t)GROUP_OOB - 65536 * 2 && N * K * 2 < (int64_t)GROUP_OOB - 65536 * 2, AQ_E_RANGE);
  auto go = [&](auto shape, auto glu_tag) -> int {
    using G = decltype(shape);
    constexpr bool GLU = decltype(glu_tag)::value;
    constexpr int cols = GLU ? G::WROWS / 2 : G::WROWS;
    const dim3 grid((unsigned)((F + cols - 1) / cols), (unsigned)(n_tiles - 1));
    grouped_mfma_kernel<G, GLU><<<grid, G::THREADS, 0, st>>>(p, (const uint16_t*)x, (const uint16_t*)w, (uint16_t*)out);
    return launched();
  };
  SQ_CHECK(tile == GroupWide::TROWS || tile == GroupNarrow::TROWS, AQ_E_SHAPE);
  if (tile == GroupWide::TROWS) return glu ? go(GroupWide{}, std::true_type{}) : go(GroupWide{}, std::false_type{});
  return glu ? go(GroupNarrow{}, std::true_type{}) : go(GroupNarrow{}, std::false_type{});
}

// whether the two launches below serve these sizes
extern "C" int aqs_moe_step_ok(int64_t M, int64_t N, int64_t F, int64_t Fs, int64_t Ex, int64_t top) {
  return M > 0 && M <= 8 && N > 0 && N % 8 == 0 && F > 0 && F % 8 == 0 && Fs >= 0 && Fs % 8 == 0 && Ex > 0 && Ex <= MAX_EXPERTS && top > 0 &&
         top <= Ex && top <= 64;
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
