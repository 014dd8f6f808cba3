// Row operations of the hybrid decoder outside its matrix products and mixers: embedding lookup into
// the fp32 residual stream, residual add + RMSNorm (with a norm of the branch in front of the sum, and routed experts'
// rows collected, where a design has them), the GLUs, and the gated norms that close the linear recurrences.
#include "seq_common.h"

namespace sq {

constexpr int ROW_THREADS = 256;

template <typename T, int V>
struct Pack {};
template <>
struct Pack<float, 4> {
  static __device__ __forceinline__ void load(const float* p, float (&o)[4]) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    o[0] = v.x, o[1] = v.y, o[2] = v.z, o[3] = v.w;
  }
  static __device__ __forceinline__ void store(float* p, const float (&o)[4]) {
    *reinterpret_cast<float4*>(p) = make_float4(o[0], o[1], o[2], o[3]);
  }
};
template <>
struct Pack<bf16, 4> {
  static __device__ __forceinline__ void load(const bf16* p, float (&o)[4]) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    o[0] = __uint_as_float(v.x << 16), o[1] = __uint_as_float(v.x & 0xffff0000u);
    o[2] = __uint_as_float(v.y << 16), o[3] = __uint_as_float(v.y & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16* p, const float (&o)[4]) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack2(o[0], o[1]), pack2(o[2], o[3]));
  }
};
template <typename T>
struct Pack<T, 1> {
  static __device__ __forceinline__ void load(const T* p, float (&o)[1]) { o[0] = to_f32(*p); }
  static __device__ __forceinline__ void store(T* p, const float (&o)[1]) { *p = from_f32<T>(o[0]); }
};

// x[m] = table[ids[m]] in fp32; ids outside the table read as zero rows
template <typename T>
__global__ __launch_bounds__(ROW_THREADS) void embed_kernel(const int64_t* ids, const T* table, float* x, int64_t K, int64_t V) {
  const int64_t m = blockIdx.x, id = ids[m];
  const bool ok = id >= 0 && id < V;
  for (int64_t k = threadIdx.x; k < K; k += ROW_THREADS) x[m * K + k] = ok ? to_f32(table[id * K + k]) : 0.0f;
}

struct AddNormArgs {
  float* x;            // [M, K]
  const int* slots;    // [M, top] rows of `routed` that belong to a token (negative: none)
  const float* post;   // weight of the branch's own norm
  const float* w;      // weight of the norm behind the sum
  int64_t ldy;
  int top, K;
  float mult, eps, w0;
};

// The branch's output t = y + sum_j routed[slots[m, j]] (either may be missing); POST: t <- t / rms(t) * post.
// x += mult * t, then out = x / sqrt(mean(x^2) + eps) * (w0 + w) (out optional).
template <typename T, int V, bool POST>
__global__ __launch_bounds__(ROW_THREADS) void add_rmsnorm_kernel(AddNormArgs p, const T* y, const T* routed, T* out) {
  extern __shared__ __align__(16) float row[];
  __shared__ float red[ROW_THREADS / 64];
  const int64_t m = blockIdx.x;
  const int K = p.K;
  float* xr = p.x + m * K;
  auto branch = [&](int k, float (&b)[V]) __attribute__((always_inline)) {
    if (y) {
      Pack<T, V>::load(y + m * p.ldy + k, b);
    } else {
#pragma unroll
      for (int i = 0; i < V; ++i) b[i] = 0.0f;
    }
    for (int j = 0; j < p.top; ++j) {
      const int s = p.slots[m * p.top + j];
      if (s < 0) continue;
      float e[V];
      Pack<T, V>::load(routed + (int64_t)s * K + k, e);
#pragma unroll
      for (int i = 0; i < V; ++i) b[i] += e[i];
    }
  };
  float ry = 1.0f, ss = 0.0f;
  if constexpr (POST) {
    for (int k = threadIdx.x * V; k < K; k += ROW_THREADS * V) {
      float b[V];
      branch(k, b);
#pragma unroll
      for (int i = 0; i < V; ++i) {
        ss += b[i] * b[i];
        row[k + i] = b[i];
      }
    }
    ss = block_sum<ROW_THREADS / 64>(ss, red);
    ry = 1.0f / sqrtf(ss / (float)K + p.eps);
    ss = 0.0f;
  }
  const bool add = POST || y || p.top;
  for (int k = threadIdx.x * V; k < K; k += ROW_THREADS * V) {
    float a[V], b[V];
    Pack<float, V>::load(xr + k, a);
    if (add) {
      if constexpr (POST) {
        float g[V];
        Pack<float, V>::load(p.post + k, g);
#pragma unroll
        for (int i = 0; i < V; ++i) b[i] = row[k + i] * ry * g[i];
      } else {
        branch(k, b);
      }
#pragma unroll
      for (int i = 0; i < V; ++i) a[i] += p.mult * b[i];
      Pack<float, V>::store(xr + k, a);
    }
#pragma unroll
    for (int i = 0; i < V; ++i) {
      ss += a[i] * a[i];
      row[k + i] = a[i];
    }
  }
  if (!out) return;
  ss = block_sum<ROW_THREADS / 64>(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)K + p.eps);
  for (int k = threadIdx.x * V; k < K; k += ROW_THREADS * V) {
    float a[V], g[V];
    Pack<float, V>::load(p.w + k, g);
#pragma unroll
    for (int i = 0; i < V; ++i) a[i] = row[k + i] * r * (p.w0 + g[i]);
    Pack<T, V>::store(out + m * K + k, a);
  }
}

// gu [M, 2F] = gate | up  ->  out [M, F]
template <typename T, int V, bool CLAMPED>
__global__ __launch_bounds__(ROW_THREADS) void glu_kernel(const T* gu, int64_t ld, float limit, T* out, int64_t M, int64_t F) {
  // one row of blocks per F, rows of the matrix in the grid's second dimension: no division
  const int64_t f = ((int64_t)blockIdx.x * ROW_THREADS + threadIdx.x) * V;
  if (f >= F) return;
  for (int64_t m = blockIdx.y; m < M; m += gridDim.y) {
    float g[V], u[V];
    Pack<T, V>::load(gu + m * ld + f, g);
    Pack<T, V>::load(gu + m * ld + F + f, u);
#pragma unroll
    for (int e = 0; e < V; ++e) g[e] = CLAMPED ? clamped_glu(g[e], u[e], limit) : silu(g[e]) * u[e];
    Pack<T, V>::store(out + m * F + f, g);
  }
}

// y [M, K] fp32 times silu(z), RMS over each of K / group consecutive parts, times w  ->  out
template <typename T>
__global__ __launch_bounds__(ROW_THREADS) void gated_group_norm_kernel(const float* y, const T* z, int64_t ldz, const float* w,
                                                                       float eps, T* out, int64_t ldo, int K, int group) {
  extern __shared__ __align__(16) float row[];
  __shared__ float red[ROW_THREADS / 64];
  const int64_t m = blockIdx.x;
  const int base = blockIdx.y * group;
  float ss = 0.0f;
  for (int k = threadIdx.x; k < group; k += ROW_THREADS) {
    const float v = y[m * K + base + k] * silu(to_f32(z[m * ldz + base + k]));
    row[k] = v;
    ss += v * v;
  }
  ss = block_sum<ROW_THREADS / 64>(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)group + eps);
  for (int k = threadIdx.x; k < group; k += ROW_THREADS)
    out[m * ldo + base + k] = from_f32<T>(row[k] * r * w[base + k]);
}

// y [M, K] fp32 over its root mean square, times w, times sigmoid(z)  ->  out
template <typename T, int V>
__global__ __launch_bounds__(ROW_THREADS) void norm_gate_kernel(const float* y, const T* z, int64_t ldz, const float* w, float eps,
                                                                T* out, int64_t ldo, int K) {
  extern __shared__ __align__(16) float row[];
  __shared__ float red[ROW_THREADS / 64];
  const int64_t m = blockIdx.x;
  float ss = 0.0f;
  for (int k = threadIdx.x * V; k < K; k += ROW_THREADS * V) {
    float a[V];
    Pack<float, V>::load(y + m * K + k, a);
#pragma unroll
    for (int i = 0; i < V; ++i) {
      ss += a[i] * a[i];
      row[k + i] = a[i];
    }
  }
  ss = block_sum<ROW_THREADS / 64>(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)K + eps);
  for (int k = threadIdx.x * V; k < K; k += ROW_THREADS * V) {
    float a[V], g[V], f[V];
    Pack<float, V>::load(w + k, g);
    Pack<T, V>::load(z + m * ldz + k, f);
#pragma unroll
    for (int i = 0; i < V; ++i) a[i] = row[k + i] * r * g[i] * sigmoid(f[i]);
    Pack<T, V>::store(out + m * ldo + k, a);
  }
}

// Every head of o [M, H, E] fp32 over its root mean square, times w [E], times sigmoid(gate), times scale -> out.
// A wavefront takes four head vectors, their loads together; NE elements of each per lane.
template <int NE, typename T>
__global__ __launch_bounds__(ROW_THREADS) void head_norm_gate_kernel(const float* o, const T* gate, int64_t ldg, const float* w,
                                                                     float eps, float scale, T* out, int64_t ldo, int64_t M,
                                                                     int H, int E) {
  constexpr int VPW = 4;
  const int lane = threadIdx.x & 63;
  // fewer than 2^26 vectors: 32-bit divisions
  const uint32_t v0 = (blockIdx.x * (ROW_THREADS / 64) + (threadIdx.x >> 6)) * VPW, nv = (uint32_t)(M * H);
  float x[VPW][NE];
  T gt[VPW][NE];
#pragma unroll
  for (int k = 0; k < VPW; ++k) {
    const uint32_t v = v0 + k < nv ? v0 + k : nv - 1, mu = v / (uint32_t)H;
    const int h = (int)(v - mu * H);
    const int64_t m = mu;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = i * 64 + lane, ec = e < E ? e : E - 1;
      x[k][i] = o[(int64_t)v * E + ec];
      gt[k][i] = gate[m * ldg + h * E + ec];
    }
  }
#pragma unroll
  for (int k = 0; k < VPW; ++k) {
    const uint32_t v = v0 + k, mu = v / (uint32_t)H;
    if (v >= nv) return;
    const int h = (int)(v - mu * H);
    const int64_t m = mu;
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < NE; ++i) ss += i * 64 + lane < E ? x[k][i] * x[k][i] : 0.0f;
    const float r = scale / sqrtf(wave_sum(ss) / (float)E + eps);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = i * 64 + lane;
      if (e < E) out[m * ldo + h * E + e] = from_f32<T>(x[k][i] * r * w[e] * sigmoid(to_f32(gt[k][i])));
    }
  }
}

}  // namespace sq

using namespace sq;

extern "C" int aqs_embed(const int64_t* ids, const void* table, int dtype, float* x, int64_t M, int64_t K, int64_t V,
                         void* stream) {
  SQ_CHECK(M >= 0 && K > 0 && V > 0, AQ_E_SHAPE);
  SQ_CHECK(M < (1 << 24), AQ_E_RANGE);  // one workgroup a row, fewer than 2^32 threads a launch
  if (M == 0) return AQ_OK;
  SQ_NEED(ids && table && x);
  SQ_DISPATCH(dtype, (embed_kernel<T><<<dim3((unsigned)M), ROW_THREADS, 0, (hipStream_t)stream>>>(ids, (const T*)table, x, K, V)));
  return launched();
}

extern "C" int aqs_add_rmsnorm(float* x, const void* y, int64_t ldy, int dtype, const void* routed, const int32_t* slots,
                               int64_t top, const float* post, float mult, const float* w, float w0, float eps, void* out, int64_t M,
                               int64_t K, void* stream) {
  SQ_CHECK(M >= 0 && K > 0 && top >= 0, AQ_E_SHAPE);
  SQ_CHECK(K <= 16384 && top <= 1024, AQ_E_RANGE);
  SQ_CHECK(!y || ldy >= K, AQ_E_SHAPE);
  SQ_CHECK(M < (1 << 24), AQ_E_RANGE);  // one workgroup a row, fewer than 2^32 threads a launch
  if (M == 0) return AQ_OK;
  const bool branch = y || top;
  SQ_NEED(x && (out || branch) && (w || !out) && (branch || !post) && (top == 0 || (routed && slots)));
  const AddNormArgs a{x, slots, post, w, ldy, (int)top, (int)K, mult, eps, w0};
  const bool v4 = K % 4 == 0 && (!y || ldy % 4 == 0) && !bad_ptr16(x) && !bad_ptr16(y) && !bad_ptr16(routed) && !bad_ptr16(post) &&
                  !bad_ptr16(w) && !bad_ptr16(out);
  const size_t lds = (size_t)K * 4;
  const dim3 grid((unsigned)M);
#define SQ_ADD(V, POST) \
  (add_rmsnorm_kernel<T, V, POST><<<grid, ROW_THREADS, lds, (hipStream_t)stream>>>(a, (const T*)y, (const T*)routed, (T*)out))
  SQ_DISPATCH(dtype, if (v4) { if (post) SQ_ADD(4, true); else SQ_ADD(4, false); }
                     else { if (post) SQ_ADD(1, true); else SQ_ADD(1, false); });
#undef SQ_ADD
  return launched();
}

static int launch_glu(const void* gu, int64_t ld, int dtype, bool clamped, float limit, void* out, int64_t M, int64_t F, void* stream) {
  SQ_CHECK(M >= 0 && F > 0 && ld >= 2 * F, AQ_E_SHAPE);
  SQ_CHECK(M < (1 << 24), AQ_E_RANGE);  // one workgroup a row, fewer than 2^32 threads a launch
  if (M == 0) return AQ_OK;
  SQ_NEED(gu && out);
  const bool v4 = F % 4 == 0 && ld % 4 == 0 && !bad_ptr16(gu) && !bad_ptr16(out);
  const int64_t nf = ((v4 ? F / 4 : F) + ROW_THREADS - 1) / ROW_THREADS;
  SQ_CHECK(nf < (1 << 20), AQ_E_RANGE);
  const dim3 grid((unsigned)nf, (unsigned)(M < 65535 ? M : 65535));
#define SQ_GLU(V, C) (glu_kernel<T, V, C><<<grid, ROW_THREADS, 0, (hipStream_t)stream>>>((const T*)gu, ld, limit, (T*)out, M, F))
  SQ_DISPATCH(dtype, if (clamped) { if (v4) SQ_GLU(4, true); else SQ_GLU(1, true); }
                     else { if (v4) SQ_GLU(4, false); else SQ_GLU(1, false); });
#undef SQ_GLU
  return launched();
}

extern "C" int aqs_clamped_glu(const void* gu, int64_t ld, int dtype, float limit, void* out, int64_t M, int64_t F, void* stream) {
  return launch_glu(gu, ld, dtype, true, limit, out, M, F, stream);
}

extern "C" int aqs_silu_glu(const void* gu, int64_t ld, int dtype, void* out, int64_t M, int64_t F, void* stream) {
  return launch_glu(gu, ld, dtype, false, 0.0f, out, M, F, stream);
}

extern "C" int aqs_norm_gate(const float* y, const void* z, int64_t ldz, int dtype, const float* w, float eps, void* out, int64_t ldo,
                             int64_t M, int64_t K, void* stream) {
  SQ_CHECK(M >= 0 && K > 0 && ldz >= K && ldo >= K, AQ_E_SHAPE);
  SQ_CHECK(K <= 16384 && M < (1 << 24), AQ_E_RANGE);
  if (M == 0) return AQ_OK;
  SQ_NEED(y && z && w && out);
  const bool v4 = K % 4 == 0 && ldz % 4 == 0 && ldo % 4 == 0 && !bad_ptr16(y) && !bad_ptr16(z) && !bad_ptr16(w) && !bad_ptr16(out);
  const size_t lds = (size_t)K * 4;
  const dim3 grid((unsigned)M);
#define SQ_NG(V) (norm_gate_kernel<T, V><<<grid, ROW_THREADS, lds, (hipStream_t)stream>>>(y, (const T*)z, ldz, w, eps, (T*)out, ldo, (int)K))
  SQ_DISPATCH(dtype, if (v4) SQ_NG(4); else SQ_NG(1));
#undef SQ_NG
  return launched();
}

extern "C" int aqs_gated_group_norm(const float* y, const void* z, int64_t ldz, int dtype, const float* w, float eps, void* out,
                                    int64_t ldo, int64_t M, int64_t K, int64_t groups, void* stream) {
  SQ_CHECK(M >= 0 && K > 0 && groups > 0 && K % groups == 0 && ldz >= K && ldo >= K, AQ_E_SHAPE);
  SQ_CHECK(K / groups <= 16384 && groups < 65536, AQ_E_RANGE);
  SQ_CHECK(M < (1 << 24), AQ_E_RANGE);  // one workgroup a row, fewer than 2^32 threads a launch
  if (M == 0) return AQ_OK;
  SQ_NEED(y && z && w && out);
  const int group = (int)(K / groups);
  SQ_DISPATCH(dtype, (gated_group_norm_kernel<T><<<dim3((unsigned)M, (unsigned)groups), ROW_THREADS, (size_t)group * 4,
                                                   (hipStream_t)stream>>>(y, (const T*)z, ldz, w, eps, (T*)out, ldo, (int)K, group)));
  return launched();
}

extern "C" int aqs_head_norm_gate(const float* o, const void* gate, int64_t ldg, int dtype, const float* w, float eps, float scale,
                                  void* out, int64_t ldo, int64_t M, int64_t H, int64_t E, void* stream) {
  SQ_CHECK(M >= 0 && H > 0 && E > 0 && ldg >= H * E && ldo >= H * E, AQ_E_SHAPE);
  SQ_CHECK(M < (1 << 24), AQ_E_RANGE);  // one workgroup a row, fewer than 2^32 threads a launch
  if (M == 0) return AQ_OK;
  SQ_NEED(o && gate && w && out);
  SQ_CHECK(M * H < (int64_t)1 << 26, AQ_E_RANGE);
  SQ_CHECK(E <= 512, AQ_E_RANGE);
  const unsigned grid = (unsigned)((M * H + 15) / 16);
#define SQ_HEADS(NE)                                                                                                       \
  (head_norm_gate_kernel<NE, T><<<grid, ROW_THREADS, 0, (hipStream_t)stream>>>(o, (const T*)gate, ldg, w, eps, scale,      \
                                                                               (T*)out, ldo, M, (int)H, (int)E))
  SQ_DISPATCH(dtype, if (E <= 64) SQ_HEADS(1); else if (E <= 128) SQ_HEADS(2); else if (E <= 256) SQ_HEADS(4); else SQ_HEADS(8));
#undef SQ_HEADS
  return launched();
}
