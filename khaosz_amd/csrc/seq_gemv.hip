// Matrix-vector products of a decode step on bf16 (or fp32) weights [N, K], for up to 8 rows of activations, with the
// row operation in front and the elementwise operation behind folded in:
//
//   in front   nothing (activations of T), RMSNorm of the fp32 residual stream, or the gated group norm that closes
//              the state-space mixer (y * silu(z), RMS per part, weight);
//   behind     bias, store as T or fp32; the clamped GLU of a gate row and its up row; x += mult * (W h) into the
//              fp32 residual stream.
//
// A workgroup of 4 wavefronts brings the rows into LDS as fp32 (every workgroup repeats the norm: the rows are a few
// KB and come from the caches), then each wavefront takes R weight rows at a time, 16 bytes per lane and row.  The first
// weights are requested before the norm, so that HBM works while the rows are being prepared.
#include "seq_common.h"

namespace sq {

enum { IN_PLAIN = 0, IN_RMSNORM = 1, IN_GATED_NORM = 2 };
enum { OUT_T = 0, OUT_F32 = 1, OUT_RESIDUAL = 2, OUT_GLU = 3 };

struct GemvArgs {
  const float* xf;    // IN_RMSNORM: x [M, K]; IN_GATED_NORM: y [M, K]
  const float* gain;  // IN_RMSNORM: w around zero; IN_GATED_NORM: plain
  const float* bias;  // [N] or null (OUT_T)
  float* res;         // OUT_RESIDUAL [M, N]
  int64_t ldx, ldz, ldo;
  int M, N, K, groups;
  int vec;            // IN_GATED_NORM: parts and z in whole 16-byte pieces
  float eps, mult, limit;
};

constexpr int GEMV_MAX_M = 8;

template <typename T, int IN, int OUT, int R, int MR>
__global__ __launch_bounds__(256) void gemv_kernel(GemvArgs p, const T* x, const T* z, const T* w, T* out) {
  // one row is kept in fp32; several as T, so that long rows fit
  using X = typename std::conditional<MR == 1, float, T>::type;
  extern __shared__ __align__(16) uint8_t xs_raw[];
  X* xs = reinterpret_cast<X*>(xs_raw);  // [M, K]
  __shared__ float red[4];
  constexpr int U = 8 / R;                      // 512-element steps of the rows in one block; the next block is in flight
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int K = p.K;
  // weight row i of this wavefront (OUT_GLU: the second half of them are the up rows of the first half)
  constexpr int OR = OUT == OUT_GLU ? R / 2 : R;  // output columns per wavefront
  const int n0 = (blockIdx.x * 4 + wave) * OR;
  const int F = OUT == OUT_GLU ? p.N / 2 : p.N;   // output columns
  const T* wr[R];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    int n = n0 + (OUT == OUT_GLU ? i % OR : i);
    n = n < F ? n : F - 1;
    wr[i] = w + (int64_t)(OUT == OUT_GLU && i >= OR ? n + F : n) * K;
  }
  Raw8<T> w0[R][U], w1[R][U];
  auto load = [&](Raw8<T> (&dst)[R][U], int k0) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + (u * 64 + lane) * 8, kc = k < K ? k : 0;
#pragma unroll
      for (int i = 0; i < R; ++i) dst[i][u].load(wr[i] + kc);
    }
  };
  load(w0, 0);
  __builtin_amdgcn_sched_barrier(0);
  // ---- rows into LDS
  for (int m = 0; m < p.M; ++m) {
    X* row = xs + m * K;
    auto put8 = [&](int k, const float* f) __attribute__((always_inline)) {
      if constexpr (std::is_same<X, float>::value) {
        reinterpret_cast<float4*>(row + k)[0] = make_float4(f[0], f[1], f[2], f[3]);
        reinterpret_cast<float4*>(row + k)[1] = make_float4(f[4], f[5], f[6], f[7]);
      } else {
        *reinterpret_cast<uint4*>(row + k) = make_uint4(pack2(f[0], f[1]), pack2(f[2], f[3]), pack2(f[4], f[5]), pack2(f[6], f[7]));
      }
    };
    if constexpr (IN == IN_PLAIN) {
      for (int k = tid * 8; k < K; k += 2048) {
        Raw8<T> v;
        v.load(x + m * p.ldx + k);
        float f[8];
        v.get(f);
        put8(k, f);
      }
    } else if constexpr (IN == IN_RMSNORM) {
      // the row stays in registers between the two passes where it fits (up to 4 pieces of 2048)
      constexpr int KEEP = 4;
      float keep[KEEP][8], ss = 0.0f;
#pragma unroll
      for (int i = 0; i < KEEP; ++i) {
        const int k = i * 2048 + tid * 8;
        if (k < K) load_vec<8>(p.xf + m * p.ldx + k, keep[i]);
        else
#pragma unroll
          for (int e = 0; e < 8; ++e) keep[i][e] = 0.0f;
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += keep[i][e] * keep[i][e];
      }
      for (int k = KEEP * 2048 + tid * 8; k < K; k += 2048) {
        float f[8];
        load_vec<8>(p.xf + m * p.ldx + k, f);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += f[e] * f[e];
      }
      ss = block_sum<4>(ss, red);
      const float r = 1.0f / sqrtf(ss / (float)K + p.eps);
      auto norm8 = [&](int k, float* f) __attribute__((always_inline)) {
        float g[8];
        load_vec<8>(p.gain + k, g);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] *= r * (1.0f + g[e]);
        put8(k, f);
      };
#pragma unroll
      for (int i = 0; i < KEEP; ++i) {
        const int k = i * 2048 + tid * 8;
        if (k < K) norm8(k, keep[i]);
      }
      for (int k = KEEP * 2048 + tid * 8; k < K; k += 2048) {
        float f[8];
        load_vec<8>(p.xf + m * p.ldx + k, f);
        norm8(k, f);
      }
    } else {
      const int part = K / p.groups;
      for (int g = 0; g < p.groups; ++g) {
        const float* yr = p.xf + m * p.ldx + g * part;
        const T* zr = z + m * p.ldz + g * part;
        const float* gr = p.gain + g * part;
        float ss = 0.0f;
        if (p.vec) {
          // 8 values at a time; the first 4 pieces of 2048 stay in registers between the two passes
          constexpr int KEEP = 4;
          float keep[KEEP][8];
          Raw8<T> zk[KEEP];
#pragma unroll
          for (int i = 0; i < KEEP; ++i) {
            const int k = i * 2048 + tid * 8, kc = k < part ? k : 0;
            if (i * 2048 < part) {  // uniform
              load_vec<8>(yr + kc, keep[i]);
              zk[i].load(zr + kc);
            }
          }
          auto gate8 = [&](float* v, const Raw8<T>& zv) __attribute__((always_inline)) {
            float f[8];
            zv.get(f);
#pragma unroll
            for (int e = 0; e < 8; ++e) {
              v[e] *= silu(f[e]);
              ss += v[e] * v[e];
            }
          };
#pragma unroll
          for (int i = 0; i < KEEP; ++i)
            if (i * 2048 + tid * 8 < part) gate8(keep[i], zk[i]);
          for (int k = KEEP * 2048 + tid * 8; k < part; k += 2048) {
            float v[8];
            Raw8<T> zv;
            load_vec<8>(yr + k, v);
            zv.load(zr + k);
            gate8(v, zv);
          }
          ss = block_sum<4>(ss, red);
          const float r = 1.0f / sqrtf(ss / (float)part + p.eps);
          auto put = [&](int k, float* v) __attribute__((always_inline)) {
            float gv[8];
            load_vec<8>(gr + k, gv);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] *= r * gv[e];
            put8(g * part + k, v);
          };
#pragma unroll
          for (int i = 0; i < KEEP; ++i)
            if (i * 2048 + tid * 8 < part) put(i * 2048 + tid * 8, keep[i]);
          for (int k = KEEP * 2048 + tid * 8; k < part; k += 2048) {
            float v[8];
            Raw8<T> zv;
            load_vec<8>(yr + k, v);
            zv.load(zr + k);
            gate8(v, zv);
            put(k, v);
          }
        } else {
          for (int k = tid; k < part; k += 256) {
            const float v = yr[k] * silu(to_f32(zr[k]));
            ss += v * v;
          }
          ss = block_sum<4>(ss, red);
          const float r = 1.0f / sqrtf(ss / (float)part + p.eps);
          for (int k = tid; k < part; k += 256) row[g * part + k] = from_f32<X>(yr[k] * silu(to_f32(zr[k])) * r * gr[k]);
        }
      }
    }
  }
  __syncthreads();
  // ---- products
  float acc[R][MR];
#pragma unroll
  for (int i = 0; i < R; ++i)
#pragma unroll
    for (int m = 0; m < MR; ++m) acc[i][m] = 0.0f;
  auto block = [&](const Raw8<T> (&ws)[R][U], int k0) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + (u * 64 + lane) * 8;
      if (k >= K) continue;
      float f[R][8];
#pragma unroll
      for (int i = 0; i < R; ++i) ws[i][u].get(f[i]);
#pragma unroll
      for (int m = 0; m < MR; ++m) {
        if (m >= p.M) break;
        float a[8];
        Raw8<X> xr;
        xr.load(xs + m * K + k);
        xr.get(a);
#pragma unroll
        for (int i = 0; i < R; ++i)
#pragma unroll
          for (int e = 0; e < 8; ++e) acc[i][m] = fmaf(f[i][e], a[e], acc[i][m]);
      }
    }
  };
  constexpr int STEP = U * 512;
  for (int k0 = 0; k0 < K; k0 += 2 * STEP) {
    if (k0 + STEP < K) load(w1, k0 + STEP);
    block(w0, k0);
    if (k0 + STEP >= K) break;
    if (k0 + 2 * STEP < K) load(w0, k0 + 2 * STEP);
    block(w1, k0 + STEP);
  }
  // ---- sums over the lanes and the output
#pragma unroll
  for (int m = 0; m < MR; ++m) {
    if (m >= p.M) break;
    float s[R];
#pragma unroll
    for (int i = 0; i < R; ++i) s[i] = wave_sum(acc[i][m]);
    if (lane != 0) continue;
#pragma unroll
    for (int i = 0; i < OR; ++i) {
      const int n = n0 + i;
      if (n >= F) break;
      if constexpr (OUT == OUT_T) out[m * p.ldo + n] = from_f32<T>(s[i] + (p.bias ? p.bias[n] : 0.0f));
      else if constexpr (OUT == OUT_F32) p.res[m * p.ldo + n] = s[i];
      else if constexpr (OUT == OUT_RESIDUAL) p.res[m * p.ldo + n] += p.mult * s[i];
      else out[m * p.ldo + n] = from_f32<T>(clamped_glu(s[i], s[i + OR], p.limit));
    }
  }
}

template <typename T, int IN, int OUT>
int launch_gemv(const GemvArgs& p, const void* x, const void* z, const void* w, void* out, hipStream_t stream) {
  const int F = OUT == OUT_GLU ? p.N / 2 : p.N;
  const size_t lds = (size_t)p.M * p.K * (p.M == 1 ? 4 : sizeof(T));
  auto go = [&](auto r_tag, auto m_tag) -> int {
    constexpr int R = decltype(r_tag)::value, MR = decltype(m_tag)::value;
    constexpr int OR = OUT == OUT_GLU ? R / 2 : R;
    auto* k = gemv_kernel<T, IN, OUT, R, MR>;
    if (lds > 64 * 1024) {
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    k<<<dim3((unsigned)((F + 4 * OR - 1) / (4 * OR))), 256, lds, stream>>>(p, (const T*)x, (const T*)z, (const T*)w, (T*)out);
    return launched();
  };
  auto rows = [&](auto m_tag) -> int {
    // two rows per wavefront once that still leaves four wavefronts per SIMD (four rows were slower: 13.6 against 10.1 us
    // for 8704 x 2048, 29.7 against 26.9 us for 16896 x 4096)
    if (OUT == OUT_GLU || F >= 4096) return go(std::integral_constant<int, 2>{}, m_tag);
    return go(std::integral_constant<int, OUT == OUT_GLU ? 2 : 1>{}, m_tag);
  };
  if (p.M == 1) return rows(std::integral_constant<int, 1>{});
  return rows(std::integral_constant<int, GEMV_MAX_M>{});
}

}  // namespace sq

using namespace sq;

extern "C" int aqs_gemv_ok(int dtype, int64_t M, int64_t N, int64_t K) {
  return M > 0 && M <= GEMV_MAX_M && N > 0 && N < (1 << 24) && K > 0 && K % 8 == 0 &&
         M * K * (M > 1 && dtype == AQ_BF16 ? 2 : 4) <= 144 * 1024;
}

// in_kind: 0 plain (x of dtype, stride ldx), 1 rmsnorm (xf, gain, eps), 2 gated group norm (xf = y, x = z with stride
// ldz, gain, eps, groups).  out_kind: 0 dtype (+ bias), 1 fp32 into res, 2 res += mult * (...), 3 clamped GLU into out.
extern "C" int aqs_gemv(int in_kind, int out_kind, int dtype, const void* x, int64_t ldx, const float* xf, const float* gain,
                        float eps, int64_t groups, const void* w, const float* bias, float mult, float limit, float* res, void* out,
                        int64_t ldo, int64_t M, int64_t N, int64_t K, void* stream) {
  SQ_CHECK(M >= 0 && N > 0 && K > 0, AQ_E_SHAPE);
  if (M == 0) return AQ_OK;
  SQ_CHECK(aqs_gemv_ok(dtype, M, N, K), AQ_E_SHAPE);
  SQ_NEED(w && (out_kind == OUT_F32 || out_kind == OUT_RESIDUAL ? (const void*)res : (const void*)out));
  SQ_CHECK(!bad_ptr16(w) && (in_kind == IN_GATED_NORM || !bad_ptr16(x)) && !bad_ptr16(xf) && !bad_ptr16(gain), AQ_E_ALIGN);
  SQ_CHECK(out_kind != OUT_GLU || N % 2 == 0, AQ_E_SHAPE);
  SQ_CHECK(ldo >= (out_kind == OUT_GLU ? N / 2 : N), AQ_E_SHAPE);
  GemvArgs p{};
  p.xf = xf, p.gain = gain, p.bias = bias, p.res = res, p.ldo = ldo;
  p.M = (int)M, p.N = (int)N, p.K = (int)K, p.groups = (int)groups, p.eps = eps, p.mult = mult, p.limit = limit;
  const void* z = nullptr;
  if (in_kind == IN_PLAIN) {
    SQ_NEED(x);
    SQ_CHECK(ldx >= K && ldx % 8 == 0, AQ_E_SHAPE);
    p.ldx = ldx;
  } else {
    SQ_NEED(xf && gain);
    p.ldx = K;
    if (in_kind == IN_GATED_NORM) {
      SQ_NEED(x);
      SQ_CHECK(groups > 0 && K % groups == 0 && ldx >= K, AQ_E_SHAPE);
      z = x, p.ldz = ldx;
      p.vec = K / groups % 8 == 0 && ldx % 8 == 0 && !bad_ptr16(x);
    }
  }
  hipStream_t st = (hipStream_t)stream;
#define SQ_GEMV(I, O) \
  if (in_kind == I && out_kind == O) SQ_DISPATCH(dtype, return (launch_gemv<T, I, O>(p, x, z, w, out, st)))
  SQ_GEMV(IN_PLAIN, OUT_T);
  SQ_GEMV(IN_PLAIN, OUT_RESIDUAL);
  SQ_GEMV(IN_RMSNORM, OUT_T);
  SQ_GEMV(IN_RMSNORM, OUT_F32);
  SQ_GEMV(IN_RMSNORM, OUT_GLU);
  SQ_GEMV(IN_GATED_NORM, OUT_RESIDUAL);
#undef SQ_GEMV
  return AQ_E_SHAPE;
}
