// Sliding-window grouped-query attention on a paged cache whose keys (D) and values (E) may differ in size.
//
//   prep      per head vector of a new token: RMS norm of q and k (plain weight), then interleaved rotation of the
//             first `rot` dimensions; q is stored, k and v go into their page slots.
//   prefill   the new tokens at positions pos .. pos + S over everything cached, matrix cores (bf16).
//   simple    the same for any sizes and for fp32: one wavefront per query and head.
//   decode    one new token per sequence: prep's work, and the attention over slices of 64 positions in separate
//             workgroups; `combine` merges the slices.
//
// Position i sees j with 0 <= i - j < window.  A head's output is multiplied by sigmoid(gate) -- one number for the head, or
// one for each element -- and a constant before it is stored.  Prompts may also attend to packed rows in which keys and
// values were formed from a shared latent (seq_latent.hip).  Positions come from device memory, so that one captured launch serves every step.
#include "seq_common.h"

namespace sq {

struct AttnDims {
  const int* pos;        // [B]
  const int64_t* table;  // [B, P]; null: packed rows, P * page of them per sequence (see page_row)
  int64_t P, n_pages;
  int S, H, G, D, E, page, window;
};

struct PrepArgs {
  AttnDims a;
  const float* q_norm;  // [D]
  const float* k_norm;
  const float* cs;      // [max_pos, rot / 2, 2] cos, sin
  int64_t ld, o_q, o_k, o_v, max_pos;
  int64_t M;
  int rot;
  float eps;
};

// Where the elements of keys and values lie.  Row r, KV head g: the key's first D0 elements at k + r * ld_k + g * k_head, the
// others (shared by all heads) at ks + r * ld_s; the value at v + r * ld_v + g * v_head.
template <typename T>
struct AttnKV {
  const T* k;
  const T* ks;
  const T* v;
  int64_t ld_k, ld_s, ld_v;
  int k_head, v_head, D0;
};
template <typename T>
AttnKV<T> paged_kv(const AttnDims& a, const void* kc, const void* vc) {
  return {(const T*)kc, nullptr, (const T*)vc, (int64_t)a.G * a.D, 0, (int64_t)a.G * a.E, a.D, a.E, a.D};
}

// Packed rows hold the positions from the block of 64 on in which the first new token's window begins.
__device__ __forceinline__ int packed_base(const AttnDims& a, int b) {
  const int lo = a.pos[b] - a.window + 1;
  return lo > 0 ? lo / 64 * 64 : 0;
}
template <typename T>
__device__ __forceinline__ int64_t page_row(const AttnDims& a, int b, int t) {
  if (!a.table) {
    const int64_t r = t - packed_base(a, b), n = a.P * a.page;
    return r >= 0 && r < n ? b * n + r : -1;
  }
  const int lp = (int)((uint32_t)t / (uint32_t)a.page);
  const int64_t phys = lp < a.P ? a.table[(int64_t)b * a.P + lp] : -1;
  return phys >= 0 && phys < a.n_pages ? phys * a.page + (t - lp * a.page) : -1;
}

// RMS norm and rotation of one head vector by one wavefront: lane l holds the NP pairs l, l + 64, ... (zeros past D)
template <int NP, typename T>
struct HeadVec {
  T raw[NP][2];
  __device__ __forceinline__ void load(const T* src, int D, int lane) {
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = 2 * (i * 64 + lane);
      raw[i][0] = src[d < D ? d : 0];
      raw[i][1] = src[d + 1 < D ? d + 1 : 0];
    }
  }
  __device__ __forceinline__ void norm_rotate(const float* w, const float* cs, int D, int rot, float eps, int lane, float (&o)[NP][2]) const {
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = 2 * (i * 64 + lane);
      o[i][0] = d < D ? to_f32(raw[i][0]) : 0.0f;
      o[i][1] = d + 1 < D ? to_f32(raw[i][1]) : 0.0f;
      ss += o[i][0] * o[i][0] + o[i][1] * o[i][1];
    }
    const float r = 1.0f / sqrtf(wave_sum(ss) / (float)D + eps);
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = 2 * (i * 64 + lane), dr = d + 1 < rot ? d : 0;
      const float u = o[i][0] * r * w[d < D ? d : 0], v = o[i][1] * r * w[d + 1 < D ? d + 1 : 0];
      const float c = rot ? cs[dr] : 1.0f, s = rot ? cs[dr + 1] : 0.0f;
      o[i][0] = d + 1 < rot ? u * c - v * s : u;
      o[i][1] = d + 1 < rot ? v * c + u * s : v;
    }
  }
};
template <int NP, typename T>
__device__ __forceinline__ void norm_rotate(const T* src, const float* w, const float* cs, int D, int rot, float eps, int lane,
                                            float (&o)[NP][2]) {
  HeadVec<NP, T> v;
  v.load(src, D, lane);
  v.norm_rotate(w, cs, D, rot, eps, lane, o);
}

constexpr int PREP_VECS = 4;  // head vectors of a token per wavefront, their loads together

// VP: value elements per lane
template <int NP, int VP, typename T>
__global__ __launch_bounds__(256) void attn_prep_kernel(PrepArgs p, const T* proj, T* q_out, T* kc, T* vc) {
  const AttnDims& a = p.a;
  const int items = a.H + 2 * a.G, groups = (items + PREP_VECS - 1) / PREP_VECS;
  const uint32_t it = blockIdx.x * 4 + (threadIdx.x >> 6), mu = it / (uint32_t)groups;  // fewer than 2^26 of them
  if (mu >= p.M) return;
  const int lane = threadIdx.x & 63, item0 = (int)(it - mu * groups) * PREP_VECS;
  const int64_t m = mu;
  const int b = (int)(mu / (uint32_t)a.S), t = a.pos[b] + (int)(mu - (uint32_t)b * a.S);
  const T* row = proj + m * p.ld;
  HeadVec<NP, T> x[PREP_VECS];
  T val[PREP_VECS][VP];
#pragma unroll
  for (int k = 0; k < PREP_VECS; ++k) {
    const int item = item0 + k < items ? item0 + k : items - 1;
    if (item < a.H + a.G) {  // uniform
      x[k].load(row + (item < a.H ? p.o_q + item * a.D : p.o_k + (item - a.H) * a.D), a.D, lane);
    } else {
      const T* src = row + p.o_v + (item - a.H - a.G) * a.E;
#pragma unroll
      for (int i = 0; i < VP; ++i) val[k][i] = src[i * 64 + lane < a.E ? i * 64 + lane : 0];
    }
  }
  const int64_t pr = page_row<T>(a, b, t);
  const float* cs = p.cs + (int64_t)(t < p.max_pos ? t : p.max_pos - 1) * p.rot;
#pragma unroll
  for (int k = 0; k < PREP_VECS; ++k) {
    const int item = item0 + k;
    if (item >= items) return;
    if (item >= a.H + a.G) {
      if (pr < 0) continue;
      T* dst = vc + (pr * a.G + item - a.H - a.G) * a.E;
#pragma unroll
      for (int i = 0; i < VP; ++i)
        if (i * 64 + lane < a.E) dst[i * 64 + lane] = val[k][i];
      continue;
    }
    const bool is_q = item < a.H;
    float o[NP][2];
    x[k].norm_rotate(is_q ? p.q_norm : p.k_norm, cs, a.D, p.rot, p.eps, lane, o);
    if (!is_q && pr < 0) continue;
    T* dst = is_q ? q_out + (m * a.H + item) * a.D : kc + (pr * a.G + item - a.H) * a.D;
#pragma unroll
    for (int i = 0; i < NP; ++i) {
      const int d = 2 * (i * 64 + lane);
      if (d < a.D) dst[d] = from_f32<T>(o[i][0]);
      if (d + 1 < a.D) dst[d + 1] = from_f32<T>(o[i][1]);
    }
  }
}

// The same where every head vector is whole 16-byte pieces: 16 lanes take a vector, 8 elements each and piece (NC pieces of
// 128), a wavefront four vectors at once.
template <typename T>
__device__ __forceinline__ void store8(T* dst, const float* v);
template <>
__device__ __forceinline__ void store8<bf16>(bf16* dst, const float* v) {
  *reinterpret_cast<uint4*>(dst) = make_uint4(pack2(v[0], v[1]), pack2(v[2], v[3]), pack2(v[4], v[5]), pack2(v[6], v[7]));
}
template <>
__device__ __forceinline__ void store8<float>(float* dst, const float* v) {
  reinterpret_cast<float4*>(dst)[0] = make_float4(v[0], v[1], v[2], v[3]);
  reinterpret_cast<float4*>(dst)[1] = make_float4(v[4], v[5], v[6], v[7]);
}
template <int NC, typename T>
__global__ __launch_bounds__(256) void attn_prep_vec_kernel(PrepArgs p, const T* proj, T* q_out, T* kc, T* vc) {
  const AttnDims& a = p.a;
  const int items = a.H + 2 * a.G, groups = (items + 3) / 4;
  const uint32_t it = blockIdx.x * 4 + (threadIdx.x >> 6), mu = it / (uint32_t)groups;  // fewer than 2^26 of them
  if (mu >= p.M) return;
  const int lane = threadIdx.x & 63, l16 = lane & 15, my = (int)(it - mu * groups) * 4 + (lane >> 4);
  const bool live = my < items;
  const int item = live ? my : items - 1;
  const int64_t m = mu;
  const int b = (int)(mu / (uint32_t)a.S), t = a.pos[b] + (int)(mu - (uint32_t)b * a.S);
  const bool is_q = item < a.H, is_v = item >= a.H + a.G;
  const int n = is_v ? a.E : a.D, g = is_q ? item : is_v ? item - a.H - a.G : item - a.H;
  const T* src = proj + m * p.ld + (is_q ? p.o_q : is_v ? p.o_v : p.o_k) + g * n;
  const float* w = is_q ? p.q_norm : p.k_norm;
  const float* cs = p.cs + (int64_t)(t < p.max_pos ? t : p.max_pos - 1) * p.rot;
  Raw8<T> raw[NC];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int d = (c * 16 + l16) * 8;
    raw[c].load(src + (d < n ? d : 0));
  }
  // cosines and sines of the lane's pairs, and the weights: requested at valid addresses whether they are used or not
  float2 turn[NC][4];
  float wv[NC][8];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int d = (c * 16 + l16) * 8;
    load_vec<8>(w + (d < a.D ? d : 0), wv[c]);
#pragma unroll
    for (int e = 0; e < 4; ++e)
      turn[c][e] = p.rot ? *reinterpret_cast<const float2*>(cs + (d + 2 * e < p.rot ? d + 2 * e : 0)) : make_float2(1.0f, 0.0f);
  }
  const int64_t pr = page_row<T>(a, b, t);
  float x[NC][8], ss = 0.0f;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    raw[c].get(x[c]);
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += (c * 16 + l16) * 8 < n ? x[c][e] * x[c][e] : 0.0f;
  }
  const float r = 1.0f / sqrtf(row16_sum(ss) / (float)a.D + p.eps);
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int d = (c * 16 + l16) * 8;
    if (d >= n || !live) continue;
    if (!is_v) {
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const float u = x[c][e] * r * wv[c][e], v = x[c][e + 1] * r * wv[c][e + 1];
        const float2 cs2 = d + e < p.rot ? turn[c][e / 2] : make_float2(1.0f, 0.0f);
        x[c][e] = u * cs2.x - v * cs2.y;
        x[c][e + 1] = v * cs2.x + u * cs2.y;
      }
    }
    if (!is_q && pr < 0) continue;
    store8<T>((is_q ? q_out + (m * a.H + g) * a.D : is_v ? vc + (pr * a.G + g) * a.E : kc + (pr * a.G + g) * a.D) + d, x[c]);
  }
}

struct AttnOut {
  const void* gate;  // T, [M, ld_gate] one number per head or (each) per element of the output, or null
  int64_t ld_gate, ldo;
  float scale;       // of the output
  bool each;
};
template <typename T>
__device__ __forceinline__ float head_factor(const AttnOut& o, int64_t m, int h) {
  return o.gate && !o.each ? o.scale * sigmoid(to_f32(reinterpret_cast<const T*>(o.gate)[m * o.ld_gate + h])) : o.scale;
}

constexpr float MASKED = -1.0e30f;
constexpr float LOG2E = 1.44269504088896341f;

// ---------------------------------------------------------------------------------------------- any sizes
constexpr int SIMPLE_MAX = 512;

template <typename T>
__global__ __launch_bounds__(256) void attn_simple_kernel(AttnDims a, AttnKV<T> kv, AttnOut o, float scale, const T* q, T* out,
                                                          int64_t M) {
  __shared__ float q_s[4][SIMPLE_MAX], p_s[4][64];
  __shared__ int row_s[4][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t v = (int64_t)blockIdx.x * 4 + wave;
  const bool live = v < M * a.H;
  const int64_t m = live ? v / a.H : 0;
  const int h = live ? (int)(v % a.H) : 0, g = h / (a.H / a.G), b = (int)(m / a.S);
  const int i = a.pos[b] + (int)(m % a.S), lo = i - a.window + 1 > 0 ? i - a.window + 1 : 0;
  for (int d = lane; d < a.D; d += 64) q_s[wave][d] = to_f32(q[(m * a.H + h) * a.D + d]) * scale;
  float acc[SIMPLE_MAX / 64], mx = MASKED, l = 0.0f;
#pragma unroll
  for (int e = 0; e < SIMPLE_MAX / 64; ++e) acc[e] = 0.0f;
  // the wavefronts of a workgroup may walk different numbers of tiles: everything below is per wavefront, LDS included
  __builtin_amdgcn_wave_barrier();
  for (int t0 = lo; live && t0 <= i; t0 += 64) {
    const int t = t0 + lane;
    const int64_t pr = t <= i ? page_row<T>(a, b, t) : -1;
    float s = t <= i ? 0.0f : -INFINITY;
    if (pr >= 0) {
      const T* k = kv.k + pr * kv.ld_k + (int64_t)g * kv.k_head;
      for (int d = 0; d < kv.D0; ++d) s = fmaf(to_f32(k[d]), q_s[wave][d], s);
      const T* ks = kv.ks + pr * kv.ld_s - kv.D0;
      for (int d = kv.D0; d < a.D; ++d) s = fmaf(to_f32(ks[d]), q_s[wave][d], s);
    }
    const float mn = fmaxf(mx, wave_max(s)), al = expf(mx - mn), pv = expf(s - mn);
    l = l * al + wave_sum(pv);
    mx = mn;
    p_s[wave][lane] = pv;
    row_s[wave][lane] = (int)pr;
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int e = 0; e < SIMPLE_MAX / 64; ++e) acc[e] *= al;
    const int n = i - t0 + 1 < 64 ? i - t0 + 1 : 64;
    for (int k = 0; k < n; ++k) {
      const int r = row_s[wave][k];
      if (r < 0) continue;
      const float w = p_s[wave][k];
      const T* vr = kv.v + (int64_t)r * kv.ld_v + (int64_t)g * kv.v_head;
#pragma unroll
      for (int e = 0; e < SIMPLE_MAX / 64; ++e)
        if (e * 64 + lane < a.E) acc[e] = fmaf(w, to_f32(vr[e * 64 + lane]), acc[e]);
    }
    __builtin_amdgcn_wave_barrier();
  }
  if (!live) return;
  const float f = head_factor<T>(o, m, h) / l;
#pragma unroll
  for (int e = 0; e < SIMPLE_MAX / 64; ++e)
    if (e * 64 + lane < a.E) {
      const float ge = o.each ? sigmoid(to_f32(((const T*)o.gate)[m * o.ld_gate + h * a.E + e * 64 + lane])) : 1.0f;
      out[m * o.ldo + h * a.E + e * 64 + lane] = from_f32<T>(acc[e] * f * ge);
    }
}

// ---------------------------------------------------------------------------------------------- prefill, matrix cores
// The arrangement of the causal kernel of attn_prefill.hip: workgroup = (128 queries, head), 4 wavefronts of 32
// queries, key blocks of 64; S^T = K Q^T and O^T = V^T P^T with v_mfma_f32_32x32x16_bf16, so that a lane keeps one
// query from its scores to its output.  Here the sizes are padded to DP and EP with zeros in LDS, key blocks run
// from the window's first to the query's own, and a page holds whole key blocks (page % 64 == 0).
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
constexpr int WQ = 128, WK = 64;

template <int DP, int EP>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DP + EP <= 320 ? 2 : 1))) void attn_window_kernel(
    AttnDims a, AttnKV<uint16_t> kv, AttnOut oo, float scale_log2e, const uint16_t* q, uint16_t* out, int B) {
  constexpr int KP = DP + 8, VP = WK + 4, DS = DP / 16, DT = EP / 32, KC = DP / 32, VC = EP / 32;
  extern __shared__ __align__(16) uint16_t lds[];
  uint16_t* ks = lds;            // [WK][KP]
  uint16_t* vt = lds + WK * KP;  // [EP][VP]
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 31, g2 = lane >> 5;
  const int S = a.S, nqb = (S + WQ - 1) / WQ, per = a.H * B;
  const int qblk = nqb - 1 - (int)blockIdx.x / per, h = ((int)blockIdx.x % per) % a.H, b = ((int)blockIdx.x % per) / a.H;
  const int kvh = h / (a.H / a.G), start = a.pos[b];
  const int q0 = qblk * WQ, qs = q0 + wave * 32 + col;         // this lane's query within the new tokens
  const int qp = start + qs, qw = start + q0 + wave * 32;      // its position; the wavefront's first
  const int64_t tok0 = (int64_t)b * S;
  const int last = start + (q0 + WQ < S ? q0 + WQ : S) - 1;    // position of the workgroup's last query
  const int first = start + q0 - a.window + 1 > 0 ? start + q0 - a.window + 1 : 0;
  const int D = a.D, E = a.E;

  uint4 qf[DS];
  {
    const uint16_t* src = q + ((tok0 + (qs < S ? qs : S - 1)) * a.H + h) * D + g2 * 8;
#pragma unroll
    for (int st = 0; st < DS; ++st)
      qf[st] = st * 16 + g2 * 8 < D ? *reinterpret_cast<const uint4*>(src + st * 16) : make_uint4(0, 0, 0, 0);
  }
  uint4 kr[KC], vr[VC];
  auto fetch = [&](int j) __attribute__((always_inline)) {
    const int64_t row0 = page_row<uint16_t>(a, b, j * WK), base = row0 >= 0 ? row0 : 0;
    const bool ok = row0 >= 0;
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int idx = c * 256 + tid, key = idx / (DP / 8), ch = idx % (DP / 8);
      const uint16_t* src = ch * 8 < kv.D0 ? kv.k + (base + key) * kv.ld_k + kvh * kv.k_head : kv.ks + (base + key) * kv.ld_s - kv.D0;
      kr[c] = ok && ch * 8 < D ? *reinterpret_cast<const uint4*>(src + ch * 8) : make_uint4(0, 0, 0, 0);
    }
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      const int ch = wave + 4 * c;
      vr[c] = ok && ch * 8 < E ? *reinterpret_cast<const uint4*>(kv.v + (base + lane) * kv.ld_v + kvh * kv.v_head + ch * 8) : make_uint4(0, 0, 0, 0);
    }
  };
  auto stage = [&](int j) __attribute__((always_inline)) {
#pragma unroll
    for (int c = 0; c < KC; ++c) {
      const int idx = c * 256 + tid, key = idx / (DP / 8), ch = idx % (DP / 8);
      *reinterpret_cast<uint4*>(&ks[key * KP + ch * 8]) = kr[c];
    }
    // V transposed, two keys per 4-byte store (neighbouring lanes swap halves).  Rows past the last position hold
    // whatever the page held before: a probability of zero must not meet a NaN there.
    const bool past = j * WK + lane > last;
    const bool odd = lane & 1;
    const uint32_t sel = odd ? 0x03020706u : 0x05040100u;
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      uint32_t* dst = reinterpret_cast<uint32_t*>(&vt[((wave + 4 * c) * 8 + (odd ? 1 : 0)) * VP + (lane & ~1)]);
      const uint32_t w[4] = {past ? 0 : vr[c].x, past ? 0 : vr[c].y, past ? 0 : vr[c].z, past ? 0 : vr[c].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const uint32_t other = (uint32_t)__builtin_amdgcn_mov_dpp((int)w[e], 0xB1, 0xf, 0xf, true);
        dst[e * VP] = __builtin_amdgcn_perm(other, w[e], sel);
      }
    }
  };

  f32x16 o[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[dt][r] = 0.0f;
  float m = MASKED, l = 0.0f;
  const int j0 = first / WK, j1 = last / WK;
  fetch(j0);
  for (int j = j0; j <= j1; ++j) {
    __syncthreads();
    stage(j);
    __syncthreads();
    if (j < j1) fetch(j + 1);
    const int kb = j * WK;
    // wavefront-uniform: every key ahead of every query, or behind every window
    if (kb > qw + 31 || kb + WK - 1 < qw - a.window + 1) continue;
    f32x16 s[2];
#pragma unroll
    for (int r = 0; r < 16; ++r) s[0][r] = s[1][r] = 0.0f;
    const uint16_t* k0 = &ks[col * KP + g2 * 8];
#pragma unroll
    for (int st = 0; st < DS; ++st) {
      const bf16x8 qv = __builtin_bit_cast(bf16x8, qf[st]);
      const uint4 f0 = *reinterpret_cast<const uint4*>(k0 + st * 16), f1 = *reinterpret_cast<const uint4*>(k0 + 32 * KP + st * 16);
      s[0] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, f0), qv, s[0], 0, 0, 0);
      s[1] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, f1), qv, s[1], 0, 0, 0);
    }
    // register r of tile kt is key kb + 32 kt + 8 (r / 4) + 4 g2 + r % 4
    const bool edge = kb + WK - 1 > qw || kb < qw + 31 - a.window + 1;
    float bm = -INFINITY;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 16; ++r) s[kt][r] *= scale_log2e;
    if (edge) {
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int t = kb + kt * 32 + 8 * (r / 4) + 4 * g2 + (r % 4);
          if (t > qp || t <= qp - a.window) s[kt][r] = -INFINITY;
        }
    }
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 16; ++r) bm = fmaxf(bm, s[kt][r]);
    bm = fmaxf(bm, __shfl_xor(bm, 32, 64));
    // the running maximum is raised only when an exponent would pass 2^8 (see attn_prefill.hip)
    const bool raise = __builtin_amdgcn_ballot_w64(bm > m + 8.0f) != 0;
    float alpha = 1.0f;
    if (raise) {
      const float mn = fmaxf(m, bm);
      alpha = __builtin_amdgcn_exp2f(m - mn);
      m = mn;
      l *= alpha;
    }
    uint4 pf[2][2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
      float pv[16];
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        pv[r] = __builtin_amdgcn_exp2f(s[kt][r] - m);
        l += pv[r];
      }
#pragma unroll
      for (int s2 = 0; s2 < 2; ++s2)
        pf[kt][s2] = make_uint4(pack2(pv[8 * s2 + 0], pv[8 * s2 + 1]), pack2(pv[8 * s2 + 2], pv[8 * s2 + 3]),
                                pack2(pv[8 * s2 + 4], pv[8 * s2 + 5]), pack2(pv[8 * s2 + 6], pv[8 * s2 + 7]));
    }
    if (raise) {
#pragma unroll
      for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[dt][r] *= alpha;
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const uint16_t* vrow = &vt[(dt * 32 + col) * VP + 4 * g2];
#pragma unroll
      for (int kk = 0; kk < 4; ++kk) {
        const uint2 lo = *reinterpret_cast<const uint2*>(vrow + kk * 16), hi = *reinterpret_cast<const uint2*>(vrow + kk * 16 + 8);
        o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, make_uint4(lo.x, lo.y, hi.x, hi.y)),
                                                        __builtin_bit_cast(bf16x8, pf[kk >> 1][kk & 1]), o[dt], 0, 0, 0);
      }
    }
  }
  l += __shfl_xor(l, 32, 64);
  if (qs >= S) return;
  const float f = head_factor<bf16>(oo, tok0 + qs, h) / l;
  uint16_t* dst = out + (tok0 + qs) * oo.ldo + (int64_t)h * E + 4 * g2;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (dt * 32 + 8 * r + 4 * g2 < E) {
        float v[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = o[dt][4 * r + i] * f;
        if (oo.each) {
          const uint2 z = *reinterpret_cast<const uint2*>((const uint16_t*)oo.gate + (tok0 + qs) * oo.ld_gate + (int64_t)h * E + 4 * g2 + dt * 32 + 8 * r);
          v[0] *= sigmoid(__uint_as_float(z.x << 16)), v[1] *= sigmoid(__uint_as_float(z.x & 0xffff0000u));
          v[2] *= sigmoid(__uint_as_float(z.y << 16)), v[3] *= sigmoid(__uint_as_float(z.y & 0xffff0000u));
        }
        *reinterpret_cast<uint2*>(dst + dt * 32 + 8 * r) = make_uint2(pack2(v[0], v[1]), pack2(v[2], v[3]));
      }
}

// ---------------------------------------------------------------------------------------------- decode
constexpr int DEC_HB = 4;   // query heads of a KV head per workgroup
constexpr int DEC_MAX = 256;

// NC: 128-dimension pieces of a key; LV: lanes that share a value row (8 dimensions each)
template <typename T, int NC, int LV>
__global__ __launch_bounds__(256) void attn_decode_kernel(PrepArgs p, float scale_log2e, const T* proj, T* kc, T* vc, float* part, int NS) {
  const AttnDims& a = p.a;
  constexpr int RPP = 64 / LV, NP = 16 / RPP;  // value rows per pass, passes over a wavefront's 16 keys
  __shared__ __align__(16) float q_s[DEC_HB][DEC_MAX];
  __shared__ __align__(16) T kn_s[DEC_MAX], vn_s[DEC_MAX];
  __shared__ float p_s[DEC_HB][64], m_s[DEC_HB], l_s[DEC_HB];
  __shared__ __align__(16) float acc_s[4][DEC_HB][LV * 8];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int per = a.H / a.G, nb = (per + DEC_HB - 1) / DEC_HB;
  int x = blockIdx.x;
  const int kvh = x % a.G;
  x /= a.G;
  const int hb = x % nb;
  x /= nb;
  const int split = x % NS, b = x / NS;
  const int pos = a.pos[b], lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  const int t0 = (lo / 64 + split) * 64;
  if (t0 > pos) return;  // uniform
  const int D = a.D, E = a.E, h0 = kvh * per + hb * DEC_HB;
  const int nh = per - hb * DEC_HB < DEC_HB ? per - hb * DEC_HB : DEC_HB;
  // the new token's projections first: they do not wait for the page table
  const T* row = proj + b * p.ld;
  HeadVec<NC, T> qraw, kraw;
  qraw.load(row + p.o_q + (h0 + (wave < nh ? wave : 0)) * D, D, lane);
  kraw.load(row + p.o_k + kvh * D, D, lane);
  // keys and values of this wavefront's 16 positions, requested at once.  64 positions lie in one page, all of whose rows
  // may be read; what lies past the sequence is masked or zeroed below.
  const int64_t pr0 = page_row<T>(a, b, t0), prc = pr0 >= 0 ? pr0 : 0;
  const int kl = lane >> 4, ch = lane & 15, vl = lane / LV, vch = lane % LV;
  Raw8<T> kreg[4][NC], vreg[NP];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int key = wave * 16 + i * 4 + kl, d = (c * 16 + ch) * 8;
      kreg[i][c].load(kc + ((prc + key) * a.G + kvh) * D + (d < D ? d : 0));
    }
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    const int key = wave * 16 + i * RPP + vl, e = vch * 8;
    vreg[i].load(vc + ((prc + key) * a.G + kvh) * E + (e < E ? e : 0));
  }
  const float* cs = p.cs + (int64_t)(pos < p.max_pos ? pos : p.max_pos - 1) * p.rot;
  float o[NC][2];
  if (wave < nh) {
    qraw.norm_rotate(p.q_norm, cs, D, p.rot, p.eps, lane, o);
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int d = 2 * (i * 64 + lane);
      q_s[wave][d] = o[i][0] * scale_log2e;  // zero past D, where the key pieces repeat the row's start
      q_s[wave][d + 1] = o[i][1] * scale_log2e;
    }
  }
  const bool has_new = pos < t0 + 64;
  if (has_new) {
    if (wave == 3) {
      kraw.norm_rotate(p.k_norm, cs, D, p.rot, p.eps, lane, o);
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        const int d = 2 * (i * 64 + lane);
        kn_s[d] = from_f32<T>(o[i][0]);
        kn_s[d + 1] = from_f32<T>(o[i][1]);
      }
    }
    if (wave == 2)
      for (int e = lane; e < DEC_MAX; e += 64) vn_s[e] = e < E ? row[p.o_v + kvh * E + e] : from_f32<T>(0.0f);
  }
#pragma unroll
  for (int i = 0; i < NP; ++i)
    if (pr0 < 0 || t0 + wave * 16 + i * RPP + vl >= pos) vreg[i].zero();
  __syncthreads();
  if (has_new) {
    const int key = pos - t0;  // the new token's row comes from LDS, and goes into its page
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int c = 0; c < NC; ++c)
        if (wave * 16 + i * 4 + kl == key && (c * 16 + ch) * 8 < D) kreg[i][c].load(&kn_s[(c * 16 + ch) * 8]);
#pragma unroll
    for (int i = 0; i < NP; ++i)
      if (wave * 16 + i * RPP + vl == key && vch * 8 < E) vreg[i].load(&vn_s[vch * 8]);
    if (hb == 0 && pr0 >= 0) {
      for (int d = tid; d < D; d += 256) kc[((pr0 + key) * a.G + kvh) * D + d] = kn_s[d];
      for (int e = tid; e < E; e += 256) vc[((pr0 + key) * a.G + kvh) * E + e] = vn_s[e];
    }
  }
  // ---- scores
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int key = wave * 16 + i * 4 + kl, t = t0 + key;
    float s[DEC_HB];
#pragma unroll
    for (int h = 0; h < DEC_HB; ++h) s[h] = 0.0f;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int d = (c * 16 + ch) * 8;
      float k[8];
      kreg[i][c].get(k);
#pragma unroll
      for (int h = 0; h < DEC_HB; ++h) {
        if (h >= nh) break;
        float qv[8];
        load_vec<8>(&q_s[h][d], qv);
#pragma unroll
        for (int e = 0; e < 8; ++e) s[h] = fmaf(k[e], qv[e], s[h]);
      }
    }
#pragma unroll
    for (int h = 0; h < DEC_HB; ++h) {
      if (h >= nh) break;
      const float v = row16_sum(s[h]);
      if (ch == 0) p_s[h][key] = t >= lo && t <= pos ? v : -INFINITY;
    }
  }
  __syncthreads();
  if (wave < nh) {
    const float s = p_s[wave][lane], mx = fmaxf(wave_max(s), MASKED), e = __builtin_amdgcn_exp2f(s - mx), sum = wave_sum(e);
    p_s[wave][lane] = e;
    if (lane == 0) m_s[wave] = mx, l_s[wave] = sum;
  }
  __syncthreads();
  // ---- values
  float acc[DEC_HB][8];
#pragma unroll
  for (int h = 0; h < DEC_HB; ++h)
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[h][e] = 0.0f;
#pragma unroll
  for (int i = 0; i < NP; ++i) {
    float v[8];
    vreg[i].get(v);
#pragma unroll
    for (int h = 0; h < DEC_HB; ++h) {
      if (h >= nh) break;
      const float w = p_s[h][wave * 16 + i * RPP + vl];
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[h][e] = fmaf(w, v[e], acc[h][e]);
    }
  }
#pragma unroll
  for (int h = 0; h < DEC_HB; ++h) {
    if (h >= nh) break;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
#pragma unroll
      for (int st = LV; st < 64; st <<= 1) acc[h][e] += __shfl_xor(acc[h][e], st, 64);
      if (vl == 0) acc_s[wave][h][vch * 8 + e] = acc[h][e];
    }
  }
  __syncthreads();
  const int PW = E + 4;  // numerators, maximum, denominator
  for (int i = tid; i < nh * E; i += 256) {
    const int h = i / E, e = i % E;
    part[(((int64_t)b * a.H + h0 + h) * NS + split) * PW + e] = (acc_s[0][h][e] + acc_s[1][h][e]) + (acc_s[2][h][e] + acc_s[3][h][e]);
  }
  if (tid < nh) {
    float* d = part + (((int64_t)b * a.H + h0 + tid) * NS + split) * PW + E;
    d[0] = m_s[tid];
    d[1] = l_s[tid];
  }
}

template <typename T>
__global__ __launch_bounds__(256) void attn_combine_kernel(AttnDims a, AttnOut o, const float* part, T* out, int NS) {
  __shared__ float w_s[256];
  __shared__ float red[4];
  const int tid = threadIdx.x, h = blockIdx.x % a.H, b = blockIdx.x / a.H;
  const int pos = a.pos[b], lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  int n = pos / 64 - lo / 64 + 1;
  n = n < NS ? n : NS;
  const int PW = a.E + 4;
  const float* src = part + ((int64_t)b * a.H + h) * NS * PW;
  // all slices' maxima, then weights 256 slices at a time
  float mx = MASKED;
  for (int i = tid; i < n; i += 256) mx = fmaxf(mx, src[(int64_t)i * PW + a.E]);
  mx = wave_max(mx);
  if ((tid & 63) == 0) red[tid >> 6] = mx;
  __syncthreads();
  mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  float den = 0.0f, num[SIMPLE_MAX / 256] = {};
  for (int i0 = 0; i0 < n; i0 += 256) {
    const int m = n - i0 < 256 ? n - i0 : 256;
    __syncthreads();
    if (tid < m) {
      const float* ml = src + (int64_t)(i0 + tid) * PW + a.E;
      const float w = __builtin_amdgcn_exp2f(ml[0] - mx);
      w_s[tid] = w;
      den += w * ml[1];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < SIMPLE_MAX / 256; ++k) {
      const int e = k * 256 + tid;
      if (e >= a.E) break;
      const float* col = src + (int64_t)i0 * PW + e;
#pragma unroll 8
      for (int i = 0; i < m; ++i) num[k] = fmaf(col[(int64_t)i * PW], w_s[i], num[k]);
    }
  }
  den = block_sum<4>(den, red);
  const float f = head_factor<T>(o, b, h) / den;
#pragma unroll
  for (int k = 0; k < SIMPLE_MAX / 256; ++k) {
    const int e = k * 256 + tid;
    if (e < a.E) out[b * o.ldo + h * a.E + e] = from_f32<T>(num[k] * f);
  }
}

int check_dims(const AttnDims& a, int64_t B) {
  SQ_CHECK(B >= 0 && a.S >= 0 && a.H > 0 && a.G > 0 && a.H % a.G == 0 && a.D > 0 && a.E > 0 && a.page > 0 && a.window > 0 &&
               a.P > 0 && a.n_pages > 0, AQ_E_SHAPE);
  SQ_CHECK(a.D <= SIMPLE_MAX && a.E <= SIMPLE_MAX && a.n_pages * a.page < ((int64_t)1 << 31) && B * a.S * (a.H + 2 * a.G) < (1 << 26), AQ_E_RANGE);
  SQ_NEED(a.pos && a.table);
  return AQ_OK;
}

}  // namespace sq

using namespace sq;

#define SQ_DIMS(B, S)                                                                                                  \
  AttnDims a{pos, table, P, n_pages, (int)(S), (int)H, (int)G, (int)D, (int)E, (int)page, (int)(window < (1 << 30) ? window : (1 << 30))}; \
  if (const int rc = check_dims(a, B)) return rc

extern "C" int aqs_attn_prep(const void* proj, int64_t ld, int64_t o_q, int64_t o_k, int64_t o_v, int dtype, const float* q_norm,
                             const float* k_norm, float eps, const float* cs, int64_t max_pos, int64_t rot, const int32_t* pos,
                             const int64_t* table, int64_t P, int64_t page, int64_t n_pages, void* q_out, void* kc, void* vc,
                             int64_t B, int64_t S, int64_t H, int64_t G, int64_t D, int64_t E, void* stream) {
  const int64_t window = 1;
  if (B * S == 0) return AQ_OK;
  SQ_DIMS(B, S);
  SQ_CHECK(rot >= 0 && rot % 2 == 0 && rot <= D && max_pos > 0, AQ_E_SHAPE);
  SQ_CHECK(o_q >= 0 && o_k >= 0 && o_v >= 0 && o_q + H * D <= ld && o_k + G * D <= ld && o_v + G * E <= ld, AQ_E_SHAPE);
  SQ_NEED(proj && q_norm && k_norm && (cs || rot == 0) && q_out && kc && vc);
  PrepArgs p{a, q_norm, k_norm, cs, ld, o_q, o_k, o_v, max_pos, B * S, (int)rot, eps};
  const int64_t groups = (H + 2 * G + PREP_VECS - 1) / PREP_VECS;
  const unsigned grid = (unsigned)((p.M * groups + 3) / 4);
  hipStream_t st = (hipStream_t)stream;
  if (D % 8 == 0 && E % 8 == 0 && D <= 256 && E <= 256 && ld % 8 == 0 && o_q % 8 == 0 && o_k % 8 == 0 && o_v % 8 == 0 && !bad_ptr16(proj) &&
      !bad_ptr16(q_out) && !bad_ptr16(kc) && !bad_ptr16(vc) && !bad_ptr16(q_norm) && !bad_ptr16(k_norm)) {
    const unsigned vgrid = (unsigned)((p.M * ((H + 2 * G + 3) / 4) + 3) / 4);
    SQ_DISPATCH(dtype, if (D <= 128 && E <= 128)(attn_prep_vec_kernel<1, T><<<vgrid, 256, 0, st>>>(p, (const T*)proj, (T*)q_out, (T*)kc, (T*)vc));
                else (attn_prep_vec_kernel<2, T><<<vgrid, 256, 0, st>>>(p, (const T*)proj, (T*)q_out, (T*)kc, (T*)vc)));
    return launched();
  }
#define SQ_PREP(NP, VP) (attn_prep_kernel<NP, VP, T><<<grid, 256, 0, st>>>(p, (const T*)proj, (T*)q_out, (T*)kc, (T*)vc))
  SQ_DISPATCH(dtype, if (D <= 128 && E <= 128) SQ_PREP(1, 2); else if (D <= 256 && E <= 256) SQ_PREP(2, 4); else SQ_PREP(4, 8));
#undef SQ_PREP
  return launched();
}

// whether the matrix-core kernel serves these sizes
extern "C" int aqs_attn_window_ok(int dtype, int64_t D, int64_t E, int64_t page) {
  return dtype == AQ_BF16 && D % 8 == 0 && E % 8 == 0 && D <= 256 && E <= 256 && page % WK == 0;
}

template <typename T>
static int launch_simple(const AttnDims& a, const AttnKV<T>& kv, const AttnOut& o, float scale, const void* q, void* out, int64_t B,
                         hipStream_t st) {
  const unsigned grid = (unsigned)((B * a.S * a.H + 3) / 4);
  attn_simple_kernel<T><<<grid, 256, 0, st>>>(a, kv, o, scale, (const T*)q, (T*)out, B * a.S);
  return launched();
}

static int launch_window(const AttnDims& a, const AttnKV<uint16_t>& kv, const AttnOut& o, float scale, const void* q, void* out,
                         int64_t B, hipStream_t st) {
  const dim3 grid((unsigned)(((a.S + WQ - 1) / WQ) * a.H * B));
  auto go = [&](auto dtag, auto etag) -> int {
    constexpr int DP = decltype(dtag)::value, EP = decltype(etag)::value;
    const size_t lds = (size_t)(WK * (DP + 8) + EP * (WK + 4)) * 2;
    auto* k = attn_window_kernel<DP, EP>;
    if (lds > 64 * 1024) {
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    k<<<grid, 256, lds, st>>>(a, kv, o, scale * LOG2E, (const uint16_t*)q, (uint16_t*)out, (int)B);
    return launched();
  };
  auto values = [&](auto dtag) -> int {
    if (a.E <= 64) return go(dtag, std::integral_constant<int, 64>{});
    if (a.E <= 128) return go(dtag, std::integral_constant<int, 128>{});
    return go(dtag, std::integral_constant<int, 256>{});
  };
  if (a.D <= 64) return values(std::integral_constant<int, 64>{});
  if (a.D <= 128) return values(std::integral_constant<int, 128>{});
  if (a.D <= 192) return values(std::integral_constant<int, 192>{});
  return values(std::integral_constant<int, 256>{});
}

extern "C" int aqs_attn_window(const void* q, const void* kc, const void* vc, int dtype, float scale, int64_t window, const void* gate,
                               int64_t ld_gate, float out_scale, const int32_t* pos, const int64_t* table, int64_t P, int64_t page,
                               int64_t n_pages, void* out, int64_t ldo, int64_t B, int64_t S, int64_t H, int64_t G, int64_t D,
                               int64_t E, int simple, void* stream) {
  if (B * S == 0) return AQ_OK;
  SQ_DIMS(B, S);
  SQ_NEED(q && kc && vc && out);
  SQ_CHECK(ldo >= H * E && (!gate || ld_gate >= H), AQ_E_SHAPE);
  const AttnOut o{gate, ld_gate, ldo, out_scale, false};
  hipStream_t st = (hipStream_t)stream;
  if (simple || !aqs_attn_window_ok(dtype, D, E, page) || ldo % 4 || bad_ptr16(q) || bad_ptr16(kc) || bad_ptr16(vc) || bad_ptr16(out))
    SQ_DISPATCH(dtype, return launch_simple<T>(a, paged_kv<T>(a, kc, vc), o, scale, q, out, B, st));
  return launch_window(a, paged_kv<uint16_t>(a, kc, vc), o, scale, q, out, B, st);
}

// Keys and values of every head, formed from a shared latent: kv [B * rows, ld_kv] holds the keys' first `dim` elements
// head by head, then the values; the keys' last `rot` elements are columns o_rot .. of packed [B * rows, ld_packed].
extern "C" int aqs_latent_window(const void* q, const void* kv, int64_t ld_kv, const void* packed, int64_t ld_packed, int64_t o_rot,
                                 int dtype, float scale, int64_t window, const void* gate, int64_t ld_gate, const int32_t* pos,
                                 int64_t rows, void* out, int64_t ldo, int64_t B, int64_t S, int64_t H, int64_t dim, int64_t rot,
                                 int64_t E, int simple, void* stream) {
  if (B * S == 0) return AQ_OK;
  SQ_CHECK(rows > 0 && rows % 64 == 0 && dim > 0 && rot >= 0, AQ_E_SHAPE);
  const int64_t D = dim + rot, G = H, P = rows / 64, page = 64, n_pages = P * B;
  const int64_t some_table[1] = {0}, *table = some_table;  // for the checks only
  SQ_DIMS(B, S);
  a.table = nullptr;
  SQ_NEED(q && kv && packed && out && gate);
  SQ_CHECK(ldo >= H * E && ld_gate >= H * E && ld_kv >= H * (dim + E) && o_rot >= 0 && ld_packed >= o_rot + rot, AQ_E_SHAPE);
  const AttnOut o{gate, ld_gate, ldo, 1.0f, true};
  hipStream_t st = (hipStream_t)stream;
  auto source = [&](auto* t) {
    using T = typename std::remove_pointer<decltype(t)>::type;
    return AttnKV<T>{(const T*)kv, (const T*)packed + o_rot, (const T*)kv + H * dim, ld_kv, ld_packed, ld_kv, (int)dim, (int)E, (int)dim};
  };
  if (simple || !aqs_attn_window_ok(dtype, D, E, page) || dim % 8 || o_rot % 8 || ld_kv % 8 || ld_packed % 8 || ldo % 4 || ld_gate % 4 ||
      bad_ptr16(q) || bad_ptr16(kv) || bad_ptr16(packed) || bad_ptr16(out) || bad_ptr16(gate))
    SQ_DISPATCH(dtype, return launch_simple<T>(a, source((T*)nullptr), o, scale, q, out, B, st));
  return launch_window(a, source((uint16_t*)nullptr), o, scale, q, out, B, st);
}

extern "C" int aqs_attn_decode_ok(int64_t D, int64_t E, int64_t page) {
  return D % 8 == 0 && E % 8 == 0 && D <= DEC_MAX && E <= DEC_MAX && page % 64 == 0;
}

// slices a step needs for this window when the sequence may hold up to `capacity` tokens
extern "C" int64_t aqs_attn_decode_slices(int64_t window, int64_t capacity) {
  const int64_t by_window = (window + 62) / 64 + 1, all = (capacity + 63) / 64;
  return by_window < all ? by_window : all;
}

// part: [B, H, slices, E + 4] floats
extern "C" int aqs_attn_decode(const void* proj, int64_t ld, int64_t o_q, int64_t o_k, int64_t o_v, int64_t o_gate, int dtype,
                               const float* q_norm, const float* k_norm, float eps, const float* cs, int64_t max_pos, int64_t rot,
                               float scale, int64_t window, float out_scale, const int32_t* pos, const int64_t* table, int64_t P,
                               int64_t page, int64_t n_pages, void* kc, void* vc, float* part, int64_t slices, void* out, int64_t ldo,
                               int64_t B, int64_t H, int64_t G, int64_t D, int64_t E, void* stream) {
  if (B == 0) return AQ_OK;
  SQ_DIMS(B, 1);
  SQ_CHECK(aqs_attn_decode_ok(D, E, page) && rot >= 0 && rot % 2 == 0 && rot <= D && max_pos > 0, AQ_E_SHAPE);
  SQ_CHECK(o_q >= 0 && o_k >= 0 && o_v >= 0 && o_q + H * D <= ld && o_k + G * D <= ld && o_v + G * E <= ld && o_gate + H <= ld, AQ_E_SHAPE);
  SQ_CHECK(slices == aqs_attn_decode_slices(window, P * page) && ldo >= H * E, AQ_E_SHAPE);
  SQ_NEED(proj && q_norm && k_norm && (cs || rot == 0) && kc && vc && part && out);
  SQ_CHECK(!bad_ptr16(kc) && !bad_ptr16(vc), AQ_E_ALIGN);
  PrepArgs p{a, q_norm, k_norm, cs, ld, o_q, o_k, o_v, max_pos, B, (int)rot, eps};
  const int64_t nb = (H / G + DEC_HB - 1) / DEC_HB, grid = B * slices * nb * G;
  SQ_CHECK(grid < (1 << 24), AQ_E_RANGE);
  hipStream_t st = (hipStream_t)stream;
#define SQ_DEC(NC, LV) \
  (attn_decode_kernel<T, NC, LV><<<dim3((unsigned)grid), 256, 0, st>>>(p, scale * LOG2E, (const T*)proj, (T*)kc, (T*)vc, part, (int)slices))
  SQ_DISPATCH(dtype,
              if (D <= 128) {
                if (E <= 64) SQ_DEC(1, 8);
                else if (E <= 128) SQ_DEC(1, 16);
                else SQ_DEC(1, 32);
              } else {
                if (E <= 64) SQ_DEC(2, 8);
                else if (E <= 128) SQ_DEC(2, 16);
                else SQ_DEC(2, 32);
              });
#undef SQ_DEC
  if (const int rc = launched()) return rc;
  SQ_DISPATCH(dtype, {
    const AttnOut o{o_gate >= 0 ? (const void*)((const T*)proj + o_gate) : nullptr, ld, ldo, out_scale, false};
    (attn_combine_kernel<T><<<dim3((unsigned)(B * H)), 256, 0, st>>>(a, o, part, (T*)out, (int)slices));
  });
  return launched();
}
