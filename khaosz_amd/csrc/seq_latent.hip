// Latent attention: queries and keys pass through low-rank latents.  A token's cache row is its normed key/value latent c
// (R elements) and one rotated key part shared by all heads (rot elements); per head the key is (W_uk c, rotated part)
// and the value W_uv c.  A query of head h is (dim unrotated, rot rotated) elements.
//
//   prep     per new token: norm of the query latent; norm of c and rotation of the shared part, into the page row.
//            For prompts the rows that any new token's window reaches are also laid out in position order (`packed`), so
//            that keys and values of all heads come from one matrix product over them (attention: seq_attn.hip).
//   rotate   the rotated part of every query head, in place.
//   absorb   one token per sequence: <W_uk c, q> = <c, W_uk^T q>, so W_uk moves to the query, and the cache rows are keys
//            as they are (and c, for the same reason, values).  The new token's page row is written by the same launch.
//   decode   the attention over page rows, slices of 64 positions (or more) in separate workgroups: on the matrix
//            cores for bf16 (16 heads share what is read), or one head per workgroup for any type.
//   output   merges the slices, applies W_uv and the output gate.
//
// Pairs of a rotation are elements i and i + rd / 2 of the first rd of the rot elements.
#include "seq_common.h"

namespace sq {

constexpr float MASKED = -1.0e30f;
constexpr float LOG2E = 1.44269504088896341f;

struct LatentArgs {
  const int* pos;        // [B]
  const int64_t* table;  // [B, P]
  int64_t P, n_pages, max_pos;
  const float* q_norm;   // [QR]
  const float* kv_norm;  // [R]
  const float* cs;       // [max_pos, rd / 2, 2]
  int64_t ld, o_q, o_kv; // the projection's row: query latent, then c and the shared key part
  int B, S, H, dim, rot, rd, R, QR, page, window;
  int rows;              // packed rows per sequence
  float eps;
};

__device__ __forceinline__ int64_t page_row(const LatentArgs& a, int b, int t) {
  const int lp = (int)((uint32_t)t / (uint32_t)a.page);
  const int64_t phys = lp < a.P ? a.table[(int64_t)b * a.P + lp] : -1;
  return phys >= 0 && phys < a.n_pages ? phys * a.page + (t - lp * a.page) : -1;
}

template <typename T, int V>
__device__ __forceinline__ void load_piece(const T* p, float (&o)[V]) {
  if constexpr (V == 8) {
    Raw8<T> r;
    r.load(p);
    r.get(o);
  } else {
    o[0] = to_f32(*p);
  }
}
template <typename T, int V>
__device__ __forceinline__ void store_piece(T* p, const float (&o)[V]) {
  if constexpr (V == 8 && std::is_same<T, bf16>::value) {
    *reinterpret_cast<uint4*>(p) = make_uint4(pack2(o[0], o[1]), pack2(o[2], o[3]), pack2(o[4], o[5]), pack2(o[6], o[7]));
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) p[i] = from_f32<T>(o[i]);
  }
}

// RMS norm of n elements by one wavefront, to one or two places
template <typename T, int V>
__device__ __forceinline__ void norm_row(const T* src, const float* w, float eps, int n, int lane, T* d0, T* d1) {
  constexpr int KEEP = V == 8 ? 3 : 8;
  float x[KEEP][V], ss = 0.0f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int k = (i * 64 + lane) * V;
    load_piece<T, V>(src + (k < n ? k : 0), x[i]);
#pragma unroll
    for (int e = 0; e < V; ++e) ss += k < n ? x[i][e] * x[i][e] : 0.0f;
  }
  for (int k = (KEEP * 64 + lane) * V; k < n; k += 64 * V) {
    float v[V];
    load_piece<T, V>(src + k, v);
#pragma unroll
    for (int e = 0; e < V; ++e) ss += v[e] * v[e];
  }
  const float r = 1.0f / sqrtf(wave_sum(ss) / (float)n + eps);
  auto put = [&](int k, float (&v)[V]) __attribute__((always_inline)) {
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] *= r * w[k + e];
    if (d0) store_piece<T, V>(d0 + k, v);
    if (d1) store_piece<T, V>(d1 + k, v);
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int k = (i * 64 + lane) * V;
    if (k < n) put(k, x[i]);
  }
  for (int k = (KEEP * 64 + lane) * V; k < n; k += 64 * V) {
    float v[V];
    load_piece<T, V>(src + k, v);
    put(k, v);
  }
}

// The cache row of a token at position t from its projection row: normed latent, rotated key part
template <typename T, int V>
__device__ __forceinline__ void kv_row(const LatentArgs& a, const T* row, int t, int lane, T* d0, T* d1) {
  norm_row<T, V>(row + a.o_kv, a.kv_norm, a.eps, a.R, lane, d0, d1);
  const T* src = row + a.o_kv + a.R;
  const float* cs = a.cs + (int64_t)(t < a.max_pos ? t : a.max_pos - 1) * a.rd;
  const int half = a.rd / 2;
  for (int i = lane; i < half; i += 64) {
    const float u = to_f32(src[i]), v = to_f32(src[i + half]), c = cs[2 * i], s = cs[2 * i + 1];
    const T x = from_f32<T>(u * c - v * s), y = from_f32<T>(v * c + u * s);
    if (d0) d0[a.R + i] = x, d0[a.R + i + half] = y;
    if (d1) d1[a.R + i] = x, d1[a.R + i + half] = y;
  }
  for (int i = a.rd + lane; i < a.rot; i += 64) {
    if (d0) d0[a.R + i] = src[i];
    if (d1) d1[a.R + i] = src[i];
  }
}

// Wavefront items: M query latents, M cache rows, then B * rows packed rows of earlier tokens (zero where none).
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_prep_kernel(LatentArgs a, const T* proj, T* cq, T* kc, T* packed) {
  const int lane = threadIdx.x & 63;
  const int64_t M = (int64_t)a.B * a.S, DK = a.R + a.rot;
  int64_t it = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (it < M) {
    norm_row<T, V>(proj + it * a.ld + a.o_q, a.q_norm, a.eps, a.QR, lane, cq + it * a.QR, (T*)nullptr);
    return;
  }
  it -= M;
  auto base = [&](int b) { const int lo = a.pos[b] - a.window + 1; return lo > 0 ? lo / 64 * 64 : 0; };
  if (it < M) {
    const int b = (int)((uint32_t)it / (uint32_t)a.S), t = a.pos[b] + (int)((uint32_t)it - (uint32_t)b * a.S);
    const int64_t pr = page_row(a, b, t), pk = packed ? t - base(b) : -1;
    kv_row<T, V>(a, proj + it * a.ld, t, lane, pr >= 0 ? kc + pr * DK : nullptr,
                 pk >= 0 && pk < a.rows ? packed + ((int64_t)b * a.rows + pk) * DK : nullptr);
    return;
  }
  it -= M;
  if (!packed || it >= (int64_t)a.B * a.rows) return;
  const int b = (int)((uint32_t)it / (uint32_t)a.rows), t = base(b) + (int)((uint32_t)it - (uint32_t)b * a.rows), pos = a.pos[b];
  if (t >= pos && t < pos + a.S) return;  // written above
  const int64_t pr = t < pos ? page_row(a, b, t) : -1;
  T* dst = packed + it * DK;
  const T* src = kc + (pr >= 0 ? pr : 0) * DK;
  for (int k = lane * V; k < DK; k += 64 * V) {
    float v[V];
    load_piece<T, V>(src + k, v);
    if (pr < 0) {
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = 0.0f;
    }
    store_piece<T, V>(dst + k, v);
  }
}

// V pairs of one query head per thread
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_rotate_kernel(LatentArgs a, T* q, int64_t n) {
  const int64_t it = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (it >= n) return;
  const uint32_t half = a.rd / 2, per = half / V;
  const uint32_t v = (uint32_t)it / per, i0 = ((uint32_t)it - v * per) * V, m = v / (uint32_t)a.H;  // v: token and head
  const int b = (int)(m / (uint32_t)a.S), t = a.pos[b] + (int)(m - (uint32_t)b * a.S);
  const float* cs = a.cs + (int64_t)(t < a.max_pos ? t : a.max_pos - 1) * a.rd + 2 * i0;
  T* p = q + (int64_t)v * (a.dim + a.rot) + a.dim + i0;
  float x[V], y[V], c[2 * V];
#pragma unroll
  for (int i = 0; i < V; ++i) x[i] = to_f32(p[i]), y[i] = to_f32(p[half + i]);
#pragma unroll
  for (int i = 0; i < 2 * V; ++i) c[i] = cs[i];
#pragma unroll
  for (int i = 0; i < V; ++i) {
    p[i] = from_f32<T>(x[i] * c[2 * i] - y[i] * c[2 * i + 1]);
    p[half + i] = from_f32<T>(y[i] * c[2 * i] + x[i] * c[2 * i + 1]);
  }
}

// ---------------------------------------------------------------------------------------------- one token per sequence
constexpr int ABS_COLS = 128;   // latent columns per workgroup
constexpr int LAT_MAX_B = 8, LAT_MAX_DIM = 512;

// q [B, H, dim + rot] -> qa [B, H, R + rot]: W_uk^T of the unrotated part, the rotated part.  The last workgroup writes the
// new tokens' page rows.  Thread: 8 columns (tid % 16), every 16th row of W_uk [H * dim, R].
template <typename T, int MB>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentArgs a, const T* proj, const T* q, const T* uk, T* kc, T* qa) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, chunks = (a.R + ABS_COLS - 1) / ABS_COLS;
  const int DK = a.R + a.rot, DQ = a.dim + a.rot;
  if ((int)blockIdx.x == a.H * chunks) {
    for (int b = wave; b < a.B; b += 4) {
      const int64_t pr = page_row(a, b, a.pos[b]);
      kv_row<T, 8>(a, proj + b * a.ld, a.pos[b], lane, pr >= 0 ? kc + pr * DK : nullptr, (T*)nullptr);
    }
    return;
  }
  __shared__ float q_s[MB][LAT_MAX_DIM];
  __shared__ float part_s[4][MB][ABS_COLS];
  const int h = blockIdx.x / chunks, c0 = (blockIdx.x % chunks) * ABS_COLS;
  const int col = c0 + (tid & 15) * 8, r0 = tid >> 4;
  const T* w = uk + (int64_t)h * a.dim * a.R + (col < a.R ? col : 0);
  constexpr int AHEAD = 8;
  Raw8<T> wr[AHEAD];
#pragma unroll
  for (int i = 0; i < AHEAD; ++i) wr[i].load(w + (int64_t)(r0 + 16 * i < a.dim ? r0 + 16 * i : 0) * a.R);
  for (int b = 0; b < a.B; ++b)
    for (int d = tid; d < a.dim; d += 256) q_s[b][d] = to_f32(q[((int64_t)b * a.H + h) * DQ + d]);
  if (c0 == 0) {
    const int half = a.rd / 2;
    for (int x = tid; x < a.B * a.rot; x += 256) {
      const int b = x / a.rot, i = x % a.rot, t = a.pos[b];
      const float* cs = a.cs + (int64_t)(t < a.max_pos ? t : a.max_pos - 1) * a.rd;
      const T* src = q + ((int64_t)b * a.H + h) * DQ + a.dim;
      float v = to_f32(src[i]);
      if (i < half) v = v * cs[2 * i] - to_f32(src[i + half]) * cs[2 * i + 1];
      else if (i < a.rd) v = v * cs[2 * (i - half)] + to_f32(src[i - half]) * cs[2 * (i - half) + 1];
      qa[((int64_t)b * a.H + h) * DK + a.R + i] = from_f32<T>(v);
    }
  }
  __syncthreads();
  float acc[MB][8];
#pragma unroll
  for (int b = 0; b < MB; ++b)
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[b][e] = 0.0f;
  for (int i0 = r0; i0 < a.dim; i0 += 16 * AHEAD) {
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const int d = i0 + 16 * i;
      if (d >= a.dim) break;
      float f[8];
      wr[i].get(f);
      if (d + 16 * AHEAD < a.dim) wr[i].load(w + (int64_t)(d + 16 * AHEAD) * a.R);
#pragma unroll
      for (int b = 0; b < MB; ++b) {
        if (b >= a.B) break;
        const float x = q_s[b][d];
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[b][e] = fmaf(f[e], x, acc[b][e]);
      }
    }
  }
#pragma unroll
  for (int b = 0; b < MB; ++b) {
    if (b >= a.B) break;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float v = acc[b][e];
      v += __shfl_xor(v, 16, 64);
      v += __shfl_xor(v, 32, 64);
      if (lane < 16) part_s[wave][b][lane * 8 + e] = v;
    }
  }
  __syncthreads();
  for (int x = tid; x < a.B * ABS_COLS; x += 256) {
    const int b = x / ABS_COLS, c = x % ABS_COLS;
    if (c0 + c < a.R)
      qa[((int64_t)b * a.H + h) * DK + c0 + c] = from_f32<T>((part_s[0][b][c] + part_s[1][b][c]) + (part_s[2][b][c] + part_s[3][b][c]));
  }
}

// One head per workgroup, any type: 16 lanes share a key, PC pieces of 4 elements each, and keep what they read of it for
// the value sum.  part [B, H, NS, R + 4]: numerators, maximum, denominator of a slice of `span` positions.
// four elements, kept as they are until they are used
template <typename T>
struct Raw4;
template <>
struct Raw4<float> {
  float4 v;
  __device__ __forceinline__ void load(const float* p) { v = *reinterpret_cast<const float4*>(p); }
  __device__ __forceinline__ void get(float* o) const { o[0] = v.x, o[1] = v.y, o[2] = v.z, o[3] = v.w; }
};
template <>
struct Raw4<bf16> {
  uint2 v;
  __device__ __forceinline__ void load(const bf16* p) { v = *reinterpret_cast<const uint2*>(p); }
  __device__ __forceinline__ void get(float* o) const {
    o[0] = __uint_as_float(v.x << 16), o[1] = __uint_as_float(v.x & 0xffff0000u);
    o[2] = __uint_as_float(v.y << 16), o[3] = __uint_as_float(v.y & 0xffff0000u);
  }
};

template <typename T, int PC>
__global__ __launch_bounds__(256) void latent_decode_any_kernel(LatentArgs a, float scale_log2e, const T* qa, const T* kc, float* part,
                                                                int NS, int span) {
  extern __shared__ __align__(16) float lds[];  // [16][PC * 64] numerators of the key groups
  __shared__ float m_s[16], l_s[16];
  const int tid = threadIdx.x, ch = tid & 15, grp = tid >> 4;
  const int h = blockIdx.x % a.H, split = (blockIdx.x / a.H) % NS, b = blockIdx.x / (a.H * NS);
  const int pos = a.pos[b], lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0, DK = a.R + a.rot;
  const int t0 = lo / 64 * 64 + split * span;
  if (t0 > pos) return;  // uniform
  const int t1 = t0 + span < pos + 1 ? t0 + span : pos + 1;
  float q[PC][4], acc[PC][4], m = MASKED, l = 0.0f;
  const T* qr = qa + ((int64_t)b * a.H + h) * DK;
#pragma unroll
  for (int c = 0; c < PC; ++c) {
    const int d = (c * 16 + ch) * 4;
    Raw4<T> x;
    x.load(qr + (d < DK ? d : 0));
    x.get(q[c]);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      q[c][e] = d < DK ? q[c][e] * scale_log2e : 0.0f;
      acc[c][e] = 0.0f;
    }
  }
  // AH keys of this group of lanes are requested together
  constexpr int AH = (sizeof(T) == 2 ? 4 : 2) / (PC > 9 ? 2 : 1);
  for (int tb = t0; tb < t1; tb += 16 * AH) {
    Raw4<T> kr[AH][PC];
    bool on[AH];
#pragma unroll
    for (int x = 0; x < AH; ++x) {
      const int t = tb + x * 16 + grp;
      const int64_t pr = t < t1 ? page_row(a, b, t) : -1;
      on[x] = pr >= 0 && t >= lo;
      const T* src = kc + (pr >= 0 ? pr : 0) * DK;
#pragma unroll
      for (int c = 0; c < PC; ++c) {
        const int d = (c * 16 + ch) * 4;
        kr[x][c].load(src + (d < DK ? d : 0));
      }
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int x = 0; x < AH; ++x) {
      float k[PC][4], s = 0.0f;
#pragma unroll
      for (int c = 0; c < PC; ++c) {
        kr[x][c].get(k[c]);
#pragma unroll
        for (int e = 0; e < 4; ++e) s = fmaf(k[c][e], q[c][e], s);
      }
      s = row16_sum(s);
      const float mn = on[x] ? fmaxf(m, s) : m, al = __builtin_amdgcn_exp2f(m - mn), w = on[x] ? __builtin_amdgcn_exp2f(s - mn) : 0.0f;
      m = mn;
      l = l * al + w;
#pragma unroll
      for (int c = 0; c < PC; ++c)
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[c][e] = fmaf(w, on[x] ? k[c][e] : 0.0f, acc[c][e] * al);
    }
  }
  if (ch == 0) m_s[grp] = m, l_s[grp] = l;
#pragma unroll
  for (int c = 0; c < PC; ++c)
    *reinterpret_cast<float4*>(&lds[grp * PC * 64 + (c * 16 + ch) * 4]) = make_float4(acc[c][0], acc[c][1], acc[c][2], acc[c][3]);
  __syncthreads();
  float mx = MASKED;
#pragma unroll
  for (int g = 0; g < 16; ++g) mx = fmaxf(mx, m_s[g]);
  float* dst = part + (((int64_t)b * a.H + h) * NS + split) * (a.R + 4);
  for (int d = tid; d < a.R; d += 256) {
    float v = 0.0f;
#pragma unroll
    for (int g = 0; g < 16; ++g) v = fmaf(lds[g * PC * 64 + d], __builtin_amdgcn_exp2f(m_s[g] - mx), v);
    dst[d] = v;
  }
  if (tid == 0) {
    float v = 0.0f;
    for (int g = 0; g < 16; ++g) v = fmaf(l_s[g], __builtin_amdgcn_exp2f(m_s[g] - mx), v);
    dst[a.R] = mx, dst[a.R + 1] = v;
  }
}

// bf16 on the matrix cores: 16 heads per workgroup, so that a cache row is read once for all of them.  Scores: every wavefront 16
// of a block's 64 positions, operands straight from memory; values: the same rows' first R elements transposed in LDS,
// every wavefront a quarter of the columns.  KS: steps of 32 along a key; RP: R padded.
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
constexpr int LAT_VP = 72, LAT_SP = 68;

template <int RP, int KS>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 2))) void latent_decode_mfma_kernel(
    LatentArgs a, float scale_log2e, const uint16_t* qa, const uint16_t* kc, float* part, int NS, int span) {
  constexpr int VC = RP / 32, NT = RP / 64;
  extern __shared__ __align__(16) uint16_t vt[];  // [RP][LAT_VP]
  __shared__ __align__(16) float s_s[16][LAT_SP];
  __shared__ __align__(16) uint16_t p_s[16][LAT_VP];
  __shared__ float m_s[16], l_s[16], al_s[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, q4 = lane >> 4;
  const int groups = (a.H + 15) / 16, h0 = (blockIdx.x % groups) * 16, split = (blockIdx.x / groups) % NS, b = blockIdx.x / (groups * NS);
  const int pos = a.pos[b], lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0, DK = a.R + a.rot;
  const int t0 = lo / 64 * 64 + split * span;
  if (t0 > pos) return;  // uniform
  const int t1 = t0 + span < pos + 1 ? t0 + span : pos + 1;
  const int nh = a.H - h0 < 16 ? a.H - h0 : 16;
  uint4 q[KS];
  {
    const uint16_t* src = qa + ((int64_t)b * a.H + h0 + (r16 < nh ? r16 : 0)) * DK;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int d = k * 32 + q4 * 8;
      q[k] = *reinterpret_cast<const uint4*>(src + (d < DK ? d : 0));
    }
  }
  f32x4 o[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) o[n] = f32x4{0, 0, 0, 0};
  if (tid < 16) m_s[tid] = MASKED, l_s[tid] = 0.0f;
  for (int tb = t0; tb < t1; tb += 64) {
    const int64_t pr0 = page_row(a, b, tb), row0 = pr0 >= 0 ? pr0 : 0;
    uint4 k[KS], v[VC];
    const uint16_t* kr = kc + (row0 + wave * 16 + r16) * DK;
#pragma unroll
    for (int i = 0; i < KS; ++i) {
      const int d = i * 32 + q4 * 8;
      k[i] = *reinterpret_cast<const uint4*>(kr + (d < DK ? d : 0));
    }
    const uint16_t* vr = kc + (row0 + lane) * DK;
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      const int d = (wave + 4 * c) * 8;
      v[c] = *reinterpret_cast<const uint4*>(vr + (d < a.R ? d : 0));
    }
    f32x4 s = {0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < KS; ++i) {
      if (i * 32 + q4 * 8 >= DK) k[i] = make_uint4(0, 0, 0, 0);  // past the row the loads repeat its start
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, q[i]), __builtin_bit_cast(bf16x8, k[i]), s, 0, 0, 0);
    }
    // column r16: position tb + wave * 16 + r16; rows 4 q4 + r: heads
    const int t = tb + wave * 16 + r16;
    const bool on = pr0 >= 0 && t >= lo && t <= pos;
#pragma unroll
    for (int r = 0; r < 4; ++r) s_s[q4 * 4 + r][wave * 16 + r16] = on ? s[r] * scale_log2e : -INFINITY;
    // values: two positions per 4-byte store (neighbouring lanes swap halves); masked rows may hold anything
    const bool off = !(pr0 >= 0 && tb + lane >= lo && tb + lane <= pos), odd = lane & 1;
    const uint32_t sel = odd ? 0x03020706u : 0x05040100u;
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      uint32_t* dst = reinterpret_cast<uint32_t*>(&vt[((wave + 4 * c) * 8 + (odd ? 1 : 0)) * LAT_VP + (lane & ~1)]);
      const uint32_t w[4] = {off ? 0 : v[c].x, off ? 0 : v[c].y, off ? 0 : v[c].z, off ? 0 : v[c].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const uint32_t other = (uint32_t)__builtin_amdgcn_mov_dpp((int)w[e], 0xB1, 0xf, 0xf, true);
        dst[e * LAT_VP] = __builtin_amdgcn_perm(other, w[e], sel);
      }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {  // heads 4 wave + i; lane: position
      const int h = wave * 4 + i;
      const float x = s_s[h][lane], old = m_s[h], mn = fmaxf(old, wave_max(x)), e = __builtin_amdgcn_exp2f(x - mn), sum = wave_sum(e);
      const float al = __builtin_amdgcn_exp2f(old - mn), l = l_s[h] * al + sum;
      p_s[h][lane] = (uint16_t)(pack2(e, e) & 0xffffu);
      if (lane == 0) m_s[h] = mn, l_s[h] = l, al_s[h] = al;
    }
    __syncthreads();
    bf16x8 pf[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) pf[kk] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const uint4*>(&p_s[r16][kk * 32 + q4 * 8]));
#pragma unroll
    for (int n = 0; n < NT; ++n) {
#pragma unroll
      for (int r = 0; r < 4; ++r) o[n][r] *= al_s[q4 * 4 + r];
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const uint4 vf = *reinterpret_cast<const uint4*>(&vt[((wave * NT + n) * 16 + r16) * LAT_VP + kk * 32 + q4 * 8]);
        o[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[kk], __builtin_bit_cast(bf16x8, vf), o[n], 0, 0, 0);
      }
    }
    if (tb + 64 < t1) __syncthreads();  // the stages may be overwritten
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int h = q4 * 4 + r;
    if (h >= nh) continue;
    float* dst = part + (((int64_t)b * a.H + h0 + h) * NS + split) * (a.R + 4);
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const int d = (wave * NT + n) * 16 + r16;
      if (d < a.R) dst[d] = o[n][r];
    }
    if (wave == 0 && r16 == 0) dst[a.R] = m_s[h], dst[a.R + 1] = l_s[h];
  }
}

// Slices of head h merged, W_uv [H * E, R] applied, times sigmoid(gate [B, H * E]).  Workgroup: OUT_ROWS values of a head.
constexpr int OUT_ROWS = 32, LAT_MAX_SLICES = 64, LAT_MAX_R = 1024;

template <typename T>
__global__ __launch_bounds__(256) void latent_out_kernel(LatentArgs a, int E, const float* part, int NS, int span, const T* uv,
                                                         const T* gate, int64_t ld_gate, T* out, int64_t ldo) {
  __shared__ __align__(16) float o_s[LAT_MAX_R];
  __shared__ float w_s[LAT_MAX_SLICES];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, chunks = (E + OUT_ROWS - 1) / OUT_ROWS;
  const int h = blockIdx.x / chunks, e0 = (blockIdx.x % chunks) * OUT_ROWS + wave * (OUT_ROWS / 4), b = blockIdx.y, R = a.R;
  constexpr int PER = OUT_ROWS / 4;
  const T* w = uv + ((int64_t)h * E) * R;
  Raw8<T> wr[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) wr[i].load(w + (int64_t)(e0 + i < E ? e0 + i : 0) * R + (lane * 8 < R ? lane * 8 : 0));
  const int pos = a.pos[b], lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  int n = (pos - lo / 64 * 64) / span + 1;
  n = n < NS ? n : NS;
  const float* src = part + ((int64_t)b * a.H + h) * NS * (R + 4);
  // the first slices' numerators are requested before their weights are known
  constexpr int PRE = 16;
  float pre[2][PRE];
#pragma unroll
  for (int c = 0; c < 2; ++c)
#pragma unroll
    for (int i = 0; i < PRE; ++i) pre[c][i] = src[(int64_t)(i < n ? i : 0) * (R + 4) + (c * 256 + tid < R ? c * 256 + tid : 0)];
  __builtin_amdgcn_sched_barrier(0);
  if (wave == 0) {
    const float* ml = src + (int64_t)(lane < n ? lane : 0) * (R + 4) + R;
    const float m = lane < n ? ml[0] : MASKED, l = ml[1], mx = wave_max(m);
    const float e = lane < n ? __builtin_amdgcn_exp2f(m - mx) : 0.0f, den = wave_sum(e * l);
    w_s[lane] = e / den;
  }
  __syncthreads();
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int d = c * 256 + tid;
    float v = 0.0f;
#pragma unroll
    for (int i = 0; i < PRE; ++i) v = fmaf(pre[c][i], w_s[i], v);  // weight zero past the last slice
    if (d >= R) break;
    for (int i = PRE; i < n; ++i) v = fmaf(src[(int64_t)i * (R + 4) + d], w_s[i], v);
    o_s[d] = v;
  }
  for (int d = 512 + tid; d < R; d += 256) {
    float v = 0.0f;
    for (int i = 0; i < n; ++i) v = fmaf(src[(int64_t)i * (R + 4) + d], w_s[i], v);
    o_s[d] = v;
  }
  __syncthreads();
  float acc[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) acc[i] = 0.0f;
  for (int k = lane * 8; k < R; k += 512) {
    float x[8];
    load_vec<8>(&o_s[k], x);
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      float f[8];
      wr[i].get(f);
      if (k + 512 < R) wr[i].load(w + (int64_t)(e0 + i < E ? e0 + i : 0) * R + k + 512);
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[i] = fmaf(f[e], x[e], acc[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const float s = wave_sum(acc[i]);
    const int e = e0 + i;
    if (lane == 0 && e < E) out[b * ldo + (int64_t)h * E + e] = from_f32<T>(s * sigmoid(to_f32(gate[b * ld_gate + (int64_t)h * E + e])));
  }
}

// blocks of 64 positions that a window can touch, in at most LAT_MAX_SLICES slices: positions per slice
inline int64_t slice_span(int64_t window, int64_t capacity) {
  const int64_t by_window = (window + 62) / 64 + 1, all = (capacity + 63) / 64, blocks = by_window < all ? by_window : all;
  return (blocks + LAT_MAX_SLICES - 1) / LAT_MAX_SLICES * 64;
}
inline int64_t slice_count(int64_t window, int64_t capacity) {
  const int64_t by_window = (window + 62) / 64 + 1, all = (capacity + 63) / 64, blocks = by_window < all ? by_window : all;
  const int64_t per = slice_span(window, capacity) / 64;
  return (blocks + per - 1) / per;
}

int check_latent(const LatentArgs& a) {
  SQ_CHECK(a.B >= 0 && a.S >= 0 && a.H > 0 && a.R > 0 && a.rot >= 0 && a.rd >= 0 && a.rd % 2 == 0 && a.rd <= a.rot && a.page > 0 && a.window > 0 &&
               a.P > 0 && a.n_pages > 0 && a.max_pos > 0 && a.dim > 0, AQ_E_SHAPE);
  SQ_CHECK(a.n_pages * a.page < ((int64_t)1 << 31) && (int64_t)a.B * a.S * a.H < ((int64_t)1 << 26), AQ_E_RANGE);
  SQ_NEED(a.pos && a.table && (a.cs || a.rd == 0));
  return AQ_OK;
}

}  // namespace sq

using namespace sq;

static LatentArgs latent_args(const int32_t* pos, const int64_t* table, int64_t P, int64_t page, int64_t n_pages, const float* cs,
                              int64_t max_pos, int64_t window, int64_t B, int64_t S, int64_t H, int64_t dim, int64_t rot, int64_t rd,
                              int64_t R) {
  LatentArgs a{};
  a.pos = pos, a.table = table, a.P = P, a.page = (int)page, a.n_pages = n_pages, a.cs = cs, a.max_pos = max_pos;
  a.window = (int)(window < (1 << 30) ? window : (1 << 30));
  a.B = (int)B, a.S = (int)S, a.H = (int)H, a.dim = (int)dim, a.rot = (int)rot, a.rd = (int)rd, a.R = (int)R;
  return a;
}

extern "C" int aqs_latent_prep(const void* proj, int64_t ld, int64_t o_q, int64_t o_kv, int dtype, const float* q_norm,
                               const float* kv_norm, float eps, const float* cs, int64_t max_pos, const int32_t* pos,
                               const int64_t* table, int64_t P, int64_t page, int64_t n_pages, int64_t window, void* cq, void* kc,
                               void* packed, int64_t rows, int64_t B, int64_t S, int64_t QR, int64_t R, int64_t rot, int64_t rd,
                               void* stream) {
  if (B * S == 0) return AQ_OK;
  LatentArgs a = latent_args(pos, table, P, page, n_pages, cs, max_pos, window, B, S, 1, 1, rot, rd, R);
  if (const int rc = check_latent(a)) return rc;
  SQ_CHECK(QR > 0 && o_q >= 0 && o_kv >= 0 && o_q + QR <= ld && o_kv + R + rot <= ld && (!packed || rows > 0), AQ_E_SHAPE);
  SQ_NEED(proj && q_norm && kv_norm && cq && kc);
  a.ld = ld, a.o_q = o_q, a.o_kv = o_kv, a.QR = (int)QR, a.q_norm = q_norm, a.kv_norm = kv_norm, a.eps = eps;
  a.rows = packed ? (int)rows : 0;
  const int64_t items = 2 * B * S + B * a.rows;
  SQ_CHECK(items < (1 << 26), AQ_E_RANGE);
  const unsigned grid = (unsigned)((items + 3) / 4);
  const bool v8 = ld % 8 == 0 && o_q % 8 == 0 && o_kv % 8 == 0 && QR % 8 == 0 && R % 8 == 0 && rot % 8 == 0 && !bad_ptr16(proj) &&
                  !bad_ptr16(cq) && !bad_ptr16(kc) && !bad_ptr16(packed);
#define SQ_PREP(V) (latent_prep_kernel<T, V><<<grid, 256, 0, (hipStream_t)stream>>>(a, (const T*)proj, (T*)cq, (T*)kc, (T*)packed))
  SQ_DISPATCH(dtype, if (v8) SQ_PREP(8); else SQ_PREP(1));
#undef SQ_PREP
  return launched();
}

extern "C" int aqs_latent_rotate(void* q, int dtype, const float* cs, int64_t max_pos, const int32_t* pos, int64_t B, int64_t S, int64_t H,
                                 int64_t dim, int64_t rot, int64_t rd, void* stream) {
  if (B * S == 0 || rd == 0) return AQ_OK;
  const int64_t unused[1] = {0};
  LatentArgs a = latent_args(pos, unused, 1, 1, 1, cs, max_pos, 1, B, S, H, dim, rot, rd, 1);
  if (const int rc = check_latent(a)) return rc;
  SQ_NEED(q);
  const bool v4 = rd / 2 % 4 == 0;
  const int64_t n = B * S * H * (rd / 2) / (v4 ? 4 : 1);
  SQ_CHECK(n < ((int64_t)1 << 31), AQ_E_RANGE);
  const unsigned grid = (unsigned)((n + 255) / 256);
#define SQ_ROT(V) (latent_rotate_kernel<T, V><<<grid, 256, 0, (hipStream_t)stream>>>(a, (T*)q, n))
  SQ_DISPATCH(dtype, if (v4) SQ_ROT(4); else SQ_ROT(1));
#undef SQ_ROT
  return launched();
}

// sizes of the one-token path
extern "C" int aqs_latent_decode_ok(int64_t B, int64_t dim, int64_t rot, int64_t R, int64_t E, int64_t page) {
  return B > 0 && B <= LAT_MAX_B && dim > 0 && dim % 8 == 0 && dim <= LAT_MAX_DIM && rot >= 0 && rot % 8 == 0 && R > 0 && R % 8 == 0 &&
         R <= LAT_MAX_R && R + rot <= 1152 && E > 0 && page % 64 == 0;
}
extern "C" int64_t aqs_latent_decode_slices(int64_t window, int64_t capacity) { return slice_count(window, capacity); }

// One token per sequence: its page row, the attention, W_uv and the gate.  q [B, H, dim + rot] before rotation;
// qa scratch of B * H * (R + rot) elements; part scratch of B * H * slices * (R + 4) floats.
extern "C" int aqs_latent_decode(const void* proj, int64_t ld, int64_t o_kv, int64_t o_gate, const void* q, const void* uk,
                                 const void* uv, int dtype, const float* kv_norm, float eps, const float* cs, int64_t max_pos,
                                 float scale, int64_t window, const int32_t* pos, const int64_t* table, int64_t P, int64_t page,
                                 int64_t n_pages, void* kc, void* qa, float* part, int64_t slices, void* out, int64_t ldo, int64_t B,
                                 int64_t H, int64_t dim, int64_t rot, int64_t rd, int64_t R, int64_t E, void* stream) {
  if (B == 0) return AQ_OK;
  LatentArgs a = latent_args(pos, table, P, page, n_pages, cs, max_pos, window, B, 1, H, dim, rot, rd, R);
  if (const int rc = check_latent(a)) return rc;
  SQ_CHECK(aqs_latent_decode_ok(B, dim, rot, R, E, page), AQ_E_SHAPE);
  SQ_CHECK(ld % 8 == 0 && o_kv >= 0 && o_kv % 8 == 0 && o_kv + R + rot <= ld && o_gate >= 0 && o_gate + H * E <= ld && ldo >= H * E, AQ_E_SHAPE);
  SQ_CHECK(slices == slice_count(window, P * page), AQ_E_SHAPE);
  SQ_NEED(proj && q && uk && uv && kv_norm && kc && qa && part && out);
  SQ_CHECK(!bad_ptr16(proj) && !bad_ptr16(uk) && !bad_ptr16(uv) && !bad_ptr16(kc) && !bad_ptr16(qa), AQ_E_ALIGN);
  a.ld = ld, a.o_kv = o_kv, a.kv_norm = kv_norm, a.eps = eps;
  hipStream_t st = (hipStream_t)stream;
  const int span = (int)slice_span(window, P * page), NS = (int)slices, DK = (int)(R + rot);
  const int64_t chunks = (R + ABS_COLS - 1) / ABS_COLS, outs = (E + OUT_ROWS - 1) / OUT_ROWS;
  SQ_CHECK(H * chunks < (1 << 22) && B * H * slices < (1 << 24) && H * outs < (1 << 22), AQ_E_RANGE);
  const unsigned agrid = (unsigned)(H * chunks + 1);
  SQ_DISPATCH(dtype, if (B == 1)(latent_absorb_kernel<T, 1><<<agrid, 256, 0, st>>>(a, (const T*)proj, (const T*)q, (const T*)uk, (T*)kc, (T*)qa));
              else (latent_absorb_kernel<T, LAT_MAX_B><<<agrid, 256, 0, st>>>(a, (const T*)proj, (const T*)q, (const T*)uk, (T*)kc, (T*)qa)));
  if (const int rc = launched()) return rc;
  const unsigned dgrid = (unsigned)(B * H * slices);
  auto any = [&](auto tag, auto* t) -> int {
    using T = typename std::remove_pointer<decltype(t)>::type;
    constexpr int PC = decltype(tag)::value;
    auto* k = latent_decode_any_kernel<T, PC>;
    const size_t lds = (size_t)16 * PC * 64 * 4;
    if (lds > 64 * 1024) {
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    k<<<dgrid, 256, lds, st>>>(a, scale * LOG2E, (const T*)qa, (const T*)kc, part, NS, span);
    return launched();
  };
  auto pieces = [&](auto* t) -> int {
    if (DK <= 128) return any(std::integral_constant<int, 2>{}, t);
    if (DK <= 256) return any(std::integral_constant<int, 4>{}, t);
    if (DK <= 576) return any(std::integral_constant<int, 9>{}, t);
    return any(std::integral_constant<int, 18>{}, t);
  };
  auto cores = [&](auto r_tag, auto k_tag) -> int {
    constexpr int RP = decltype(r_tag)::value, KS = decltype(k_tag)::value;
    auto* k = latent_decode_mfma_kernel<RP, KS>;
    constexpr size_t lds = (size_t)RP * LAT_VP * 2;
    if (lds > 48 * 1024) {  // besides what the kernel declares
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    k<<<dim3((unsigned)(B * ((H + 15) / 16) * slices)), 256, lds, st>>>(a, scale * LOG2E, (const uint16_t*)qa, (const uint16_t*)kc, part, NS, span);
    return launched();
  };
  using std::integral_constant;
  int rc = AQ_OK;
  // a few heads in all are faster with a workgroup each (8.6 against 12.5 us for 16 heads over 1024 positions, one sequence)
  if (dtype == AQ_BF16 && R <= 512 && rot <= 128 && B * H > 16) {
    if (R <= 64) rc = cores(integral_constant<int, 64>{}, integral_constant<int, 6>{});
    else if (R <= 128) rc = cores(integral_constant<int, 128>{}, integral_constant<int, 8>{});
    else if (R <= 256) rc = cores(integral_constant<int, 256>{}, integral_constant<int, 12>{});
    else if (DK <= 576) rc = cores(integral_constant<int, 512>{}, integral_constant<int, 18>{});
    else rc = cores(integral_constant<int, 512>{}, integral_constant<int, 20>{});
  } else {
    SQ_DISPATCH(dtype, rc = pieces((T*)nullptr));
  }
  if (rc) return rc;
  const dim3 ogrid((unsigned)(H * outs), (unsigned)B);
  SQ_DISPATCH(dtype, (latent_out_kernel<T><<<ogrid, 256, 0, st>>>(a, (int)E, part, NS, span, (const T*)uv, (const T*)proj + o_gate, ld, (T*)out, ldo)));
  return launched();
}
