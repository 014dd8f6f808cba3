// Row operations of the hybrid decoder outside its matrix products and mixers: embedding lookup into
// the fp32 residual stream, residual add + RMSNorm, the clamped GLU, and the gated norms that close
// the two linear recurrences.
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

// x += mult * y (y optional), then out = x / sqrt(mean(x^2) + eps) * (1 + w) (out optional)
template <typename T, int V>
__global__ __launch_bounds__(ROW_THREADS) void add_rmsnorm_kernel(float* x, const T* y, int64_t ldy, float mult, const float* w,
                                                                  float eps, T* out, int K) {
  extern __shared__ __align__(16) float row[];
  __shared__ float red[ROW_THREADS / 64];
  const int64_t m = blockIdx.x;
  float* xr = x + m * K;
  float ss = 0.0f;
  for (int k = threadIdx.x * V; k < K; k += ROW_THREADS * V) {
    float a[V], b[V];
    Pack<float, V>::load(xr + k, a);
    if (y) {
      Pack<T, V>::load(y + m * ldy + k, b);
#pragma unroll
      for (int i = 0; i < V; ++i) a[i] += mult * b[i];
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
  const float r = 1.0f / sqrtf(ss / (float)K + eps);
  for (int k = threadIdx.x * V; k < K; k += ROW_THREADS * V) {
    float a[V], g[V];
    Pack<float, V>::load(w + k, g);
#pragma unroll
    for (int i = 0; i < V; ++i) a[i] = row[k + i] * r * (1.0f + g[i]);
    Pack<T, V>::store(out + m * K + k, a);
  }
}

// gu [M, 2F] = gate | up  ->  out [M, F]
template <typename T, int V>
__global__ __launch_bounds__(ROW_THREADS) void glu_kernel(const T* gu, int64_t ld, float limit, T* out, int64_t M, int64_t F) {
  // one row of blocks per F, rows of the matrix in the grid's second dimension: no division
  const int64_t f = ((int64_t)blockIdx.x * ROW_THREADS + threadIdx.x) * V;
  if (f >= F) return;
  for (int64_t m = blockIdx.y; m < M; m += gridDim.y) {
    float g[V], u[V];
    Pack<T, V>::load(gu + m * ld + f, g);
    Pack<T, V>::load(gu + m * ld + F + f, u);
#pragma unroll
    for (int e = 0; e < V; ++e) g[e] = clamped_glu(g[e], u[e], limit);
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

extern "C" int aqs_add_rmsnorm(float* x, const void* y, int64_t ldy, int dtype, float mult, const float* w, float eps,
                               void* out, int64_t M, int64_t K, void* stream) {
  SQ_CHECK(M >= 0 && K > 0, AQ_E_SHAPE);
  SQ_CHECK(K <= 16384, AQ_E_RANGE);
  SQ_CHECK(!y || ldy >= K, AQ_E_SHAPE);
  SQ_CHECK(M < (1 << 24), AQ_E_RANGE);  // one workgroup a row, fewer than 2^32 threads a launch
  if (M == 0) return AQ_OK;
  SQ_NEED(x && (out || y) && (w || !out));
  const bool v4 = K % 4 == 0 && ldy % 4 == 0 && !bad_ptr16(x) && !bad_ptr16(y) && !bad_ptr16(w) && !bad_ptr16(out);
  const size_t lds = (size_t)K * 4;
  const dim3 grid((unsigned)M);
  SQ_DISPATCH(dtype, if (v4)(add_rmsnorm_kernel<T, 4><<<grid, ROW_THREADS, lds, (hipStream_t)stream>>>(
                         x, (const T*)y, ldy, mult, w, eps, (T*)out, (int)K));
              else (add_rmsnorm_kernel<T, 1><<<grid, ROW_THREADS, lds, (hipStream_t)stream>>>(x, (const T*)y, ldy, mult, w, eps,
                                                                                               (T*)out, (int)K)));
  return launched();
}

extern "C" int aqs_clamped_glu(const void* gu, int64_t ld, int dtype, float limit, void* out, int64_t M, int64_t F,
                               void* stream) {
  SQ_CHECK(M >= 0 && F > 0 && ld >= 2 * F, AQ_E_SHAPE);
  SQ_CHECK(M < (1 << 24), AQ_E_RANGE);  // one workgroup a row, fewer than 2^32 threads a launch
  if (M == 0) return AQ_OK;
  SQ_NEED(gu && out);
  const bool v4 = F % 4 == 0 && ld % 4 == 0 && !bad_ptr16(gu) && !bad_ptr16(out);
  const int64_t nf = ((v4 ? F / 4 : F) + ROW_THREADS - 1) / ROW_THREADS;
  SQ_CHECK(nf < (1 << 20), AQ_E_RANGE);
  const dim3 grid((unsigned)nf, (unsigned)(M < 65535 ? M : 65535));
  SQ_DISPATCH(dtype, if (v4)(glu_kernel<T, 4><<<grid, ROW_THREADS, 0, (hipStream_t)stream>>>((const T*)gu, ld, limit, (T*)out, M, F));
              else (glu_kernel<T, 1><<<grid, ROW_THREADS, 0, (hipStream_t)stream>>>((const T*)gu, ld, limit, (T*)out, M, F)));
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
