// Matrix-vector products of a decode step on bf16 (or fp32) weights [N, K], for up to 8 rows of activations, with the
// row operation in front and the elementwise operation behind folded in:
//
//   in front   nothing (activations of T); RMSNorm of the fp32 residual stream, or of rows of T; RMSNorm of the stream
//              after a pending branch output passed its own norm and was added (the sum is stored as well, elsewhere:
//              other workgroups still read the old stream); the gated norms that close the recurrences (y * silu(z)
//              normed per part, or y normed and multiplied by sigmoid(z));
//   behind     bias, store as T or fp32; the GLU of a gate row and its up row; x += mult * (W h) into the fp32
//              residual stream; the scores of a router (fp32) beside the GLU of a shared expert.
//
// A workgroup of 4 wavefronts brings the rows into LDS (every workgroup repeats the norm: the rows are a few KB and
// come from the caches), then each wavefront takes R weight rows at a time, 16 bytes per lane and row.  The first
// weights are requested before the norm, so that HBM works while the rows are being prepared.  One row is prepared by
// the whole workgroup; of several, each wavefront prepares its own, without barriers.
#include "seq_common.h"

namespace sq {

enum { IN_PLAIN = 0, IN_RMSNORM = 1, IN_GATED_NORM = 2, IN_POST_RMSNORM = 3, IN_ROW_NORM = 4, IN_NORM_GATE = 5 };
enum { OUT_T = 0, OUT_F32 = 1, OUT_RESIDUAL = 2, OUT_GLU = 3, OUT_ROUTER_GLU = 4 };

struct GemvArgs {
  const float* xf;    // IN_(POST_)RMSNORM: x [M, K]; IN_GATED_NORM, IN_NORM_GATE: y [M, K]
  const float* gain;  // IN_(POST_)RMSNORM: w, gain0 is added to it; otherwise plain
  const float* yf;    // IN_POST_RMSNORM: the pending branch output [M, K], fp32
  const float* post;  // IN_POST_RMSNORM: the branch norm's weight
  float* x_out;       // IN_POST_RMSNORM: the new stream
  const float* bias;  // [N] or null (OUT_T)
  float* res;         // OUT_RESIDUAL, OUT_F32 [M, N]; OUT_ROUTER_GLU [M, routers]
  int64_t ldx, ldz, ldo;
  int M, N, K, groups;
  int vec;            // IN_GATED_NORM: parts and z in whole 16-byte pieces
  int routers;        // OUT_ROUTER_GLU: rows of w that are scores
  float eps, mult, limit, gain0;
};

constexpr int GEMV_MAX_M = 8;

template <typename T, int IN, int OUT, int R, int MR>
__global__ __launch_bounds__(256) void gemv_kernel(GemvArgs p, const T* x, const T* z, const T* w, T* out, T* h_out) {
  // one row is kept in fp32; several as T, so that long rows fit
  using X = typename std::conditional<MR == 1, float, T>::type;
  extern __shared__ __align__(16) uint8_t xs_raw[];
  X* xs = reinterpret_cast<X*>(xs_raw);  // [M, K]
  __shared__ float red[4];
  constexpr bool GLU = OUT == OUT_GLU || OUT == OUT_ROUTER_GLU;
  constexpr int U = 8 / R;                      // 512-element steps of the rows in one block; the next block is in flight
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int K = p.K;
  // weight row i of this wavefront (GLUs: the second half of them are the up rows of the first half)
  constexpr int OR = GLU ? R / 2 : R;             // output columns per wavefront
  const int unit = blockIdx.x * 4 + wave;
  const int nr = OUT == OUT_ROUTER_GLU ? (p.routers + R - 1) / R : 0;  // wavefronts that take R score rows
  const bool router = OUT == OUT_ROUTER_GLU && unit < nr;
  const int n0 = router ? unit * R : (unit - nr) * OR;
  const int F = OUT == OUT_ROUTER_GLU ? (p.N - p.routers) / 2 : GLU ? p.N / 2 : p.N;  // output columns
  const T* wr[R];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    if (router) {
      wr[i] = w + (int64_t)(n0 + i < p.routers ? n0 + i : p.routers - 1) * K;
    } else {
      int n = n0 + (GLU ? i % OR : i);
      n = n < F ? n : F - 1;
      wr[i] = w + (int64_t)((OUT == OUT_ROUTER_GLU ? p.routers : 0) + (GLU && i >= OR ? n + F : n)) * K;
    }
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
  // ---- rows into LDS: one row by the whole workgroup, several by a wavefront each
  constexpr int GT = MR == 1 ? 256 : 64, PIECE = GT * 8;
  constexpr int KEEP = 4;  // pieces of a row that stay in registers between the passes
  const int gid = MR == 1 ? tid : lane;
  auto gsum = [&](float v) __attribute__((always_inline)) -> float {
    if constexpr (MR == 1) return block_sum<4>(v, red);
    else return wave_sum(v);
  };
  for (int m = MR == 1 ? 0 : wave; m < p.M; m += MR == 1 ? 1 : 4) {
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
      for (int k = gid * 8; k < K; k += PIECE) {
        Raw8<T> v;
        v.load(x + m * p.ldx + k);
        float f[8];
        v.get(f);
        put8(k, f);
      }
    } else if constexpr (IN != IN_GATED_NORM) {
      // Three ways to the value that is normed, one way on: keep[] holds the first pieces, the others are formed again.
      float keep[KEEP][8], ss = 0.0f, ry = 0.0f;
      auto zero8 = [&](float* f) __attribute__((always_inline)) {
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = 0.0f;
      };
      auto load8 = [&](int k, float* f) __attribute__((always_inline)) {
        float v[8];
        if constexpr (IN == IN_ROW_NORM) {
          Raw8<T> r;
          r.load(x + m * p.ldx + k);
          r.get(v);
        } else {
          load_vec<8>(p.xf + m * p.ldx + k, v);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = v[e];
      };
      auto sum8 = [&](const float* f) __attribute__((always_inline)) {
#pragma unroll
        for (int e = 0; e < 8; ++e) ss += f[e] * f[e];
      };
#pragma unroll
      for (int i = 0; i < KEEP; ++i) {
        const int k = i * PIECE + gid * 8;
        if (k < K) load8(k, keep[i]);
        else zero8(keep[i]);
      }
      if constexpr (IN == IN_POST_RMSNORM) {
        float pend[KEEP][8];
        const float* yr = p.yf + (int64_t)m * K;
#pragma unroll
        for (int i = 0; i < KEEP; ++i) {
          const int k = i * PIECE + gid * 8;
          if (k < K) {
            float v[8];
            load_vec<8>(yr + k, v);
#pragma unroll
            for (int e = 0; e < 8; ++e) pend[i][e] = v[e];
          } else {
            zero8(pend[i]);
          }
          sum8(pend[i]);
        }
        for (int k = KEEP * PIECE + gid * 8; k < K; k += PIECE) {
          float v[8];
          load_vec<8>(yr + k, v);
          sum8(v);
        }
        ry = p.mult / sqrtf(gsum(ss) / (float)K + p.eps);
        ss = 0.0f;
        auto join = [&](int k, float* f, const float* yv) __attribute__((always_inline)) {
          float g[8];
          load_vec<8>(p.post + k, g);
#pragma unroll
          for (int e = 0; e < 8; ++e) f[e] += ry * yv[e] * g[e];
          if (blockIdx.x == 0) {
            float* xo = p.x_out + (int64_t)m * K + k;
            reinterpret_cast<float4*>(xo)[0] = make_float4(f[0], f[1], f[2], f[3]);
            reinterpret_cast<float4*>(xo)[1] = make_float4(f[4], f[5], f[6], f[7]);
          }
          sum8(f);
        };
#pragma unroll
        for (int i = 0; i < KEEP; ++i) {
          const int k = i * PIECE + gid * 8;
          if (k < K) join(k, keep[i], pend[i]);
        }
        for (int k = KEEP * PIECE + gid * 8; k < K; k += PIECE) {
          float f[8], yv[8];
          load8(k, f);
          load_vec<8>(yr + k, yv);
          join(k, f, yv);
        }
      } else {
#pragma unroll
        for (int i = 0; i < KEEP; ++i) sum8(keep[i]);
        for (int k = KEEP * PIECE + gid * 8; k < K; k += PIECE) {
          float f[8];
          load8(k, f);
          sum8(f);
        }
      }
      const float r = 1.0f / sqrtf(gsum(ss) / (float)K + p.eps);
      auto norm8 = [&](int k, float* f) __attribute__((always_inline)) {
        float g[8];
        load_vec<8>(p.gain + k, g);
        if constexpr (IN == IN_NORM_GATE) {
          Raw8<T> zv;
          zv.load(z + m * p.ldz + k);
          float q[8];
          zv.get(q);
#pragma unroll
          for (int e = 0; e < 8; ++e) f[e] *= r * g[e] * sigmoid(q[e]);
        } else {
          const float g0 = IN == IN_ROW_NORM ? 0.0f : p.gain0;
#pragma unroll
          for (int e = 0; e < 8; ++e) f[e] *= r * (g0 + g[e]);
        }
        put8(k, f);
        if constexpr (OUT == OUT_ROUTER_GLU) {
          if (blockIdx.x == 0) {
            T* ho = h_out + (int64_t)m * K + k;
#pragma unroll
            for (int e = 0; e < 8; ++e) ho[e] = from_f32<T>(f[e]);
          }
        }
      };
#pragma unroll
      for (int i = 0; i < KEEP; ++i) {
        const int k = i * PIECE + gid * 8;
        if (k < K) norm8(k, keep[i]);
      }
      for (int k = KEEP * PIECE + gid * 8; k < K; k += PIECE) {
        float f[8];
        load8(k, f);
        if constexpr (IN == IN_POST_RMSNORM) {
          float g[8], yv[8];
          load_vec<8>(p.post + k, g);
          load_vec<8>(p.yf + (int64_t)m * K + k, yv);
#pragma unroll
          for (int e = 0; e < 8; ++e) f[e] += ry * yv[e] * g[e];
        }
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
          // 8 values at a time
          float keep[KEEP][8];
          Raw8<T> zk[KEEP];
#pragma unroll
          for (int i = 0; i < KEEP; ++i) {
            const int k = i * PIECE + gid * 8, kc = k < part ? k : 0;
            if (i * PIECE < part) {  // uniform
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
            if (i * PIECE + gid * 8 < part) gate8(keep[i], zk[i]);
          for (int k = KEEP * PIECE + gid * 8; k < part; k += PIECE) {
            float v[8];
            Raw8<T> zv;
            load_vec<8>(yr + k, v);
            zv.load(zr + k);
            gate8(v, zv);
          }
          ss = gsum(ss);
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
            if (i * PIECE + gid * 8 < part) put(i * PIECE + gid * 8, keep[i]);
          for (int k = KEEP * PIECE + gid * 8; k < part; k += PIECE) {
            float v[8];
            Raw8<T> zv;
            load_vec<8>(yr + k, v);
            zv.load(zr + k);
            gate8(v, zv);
            put(k, v);
          }
        } else {
          for (int k = gid; k < part; k += GT) {
            const float v = yr[k] * silu(to_f32(zr[k]));
            ss += v * v;
          }
          ss = gsum(ss);
          const float r = 1.0f / sqrtf(ss / (float)part + p.eps);
          for (int k = gid; k < part; k += GT) row[g * part + k] = from_f32<X>(yr[k] * silu(to_f32(zr[k])) * r * gr[k]);
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
    if (router) {
#pragma unroll
      for (int i = 0; i < R; ++i)
        if (n0 + i < p.routers) p.res[m * p.routers + n0 + i] = s[i];
      continue;
    }
#pragma unroll
    for (int i = 0; i < OR; ++i) {
      const int n = n0 + i;
      if (n >= F) break;
      if constexpr (OUT == OUT_T) out[m * p.ldo + n] = from_f32<T>(s[i] + (p.bias ? p.bias[n] : 0.0f));
      else if constexpr (OUT == OUT_F32) p.res[m * p.ldo + n] = s[i];
      else if constexpr (OUT == OUT_RESIDUAL) p.res[m * p.ldo + n] += p.mult * s[i];
      else if constexpr (OUT == OUT_GLU) out[m * p.ldo + n] = from_f32<T>(clamped_glu(s[i], s[i + OR], p.limit));
      else out[m * p.ldo + n] = from_f32<T>(silu(s[i]) * s[i + OR]);
    }
  }
}

template <typename T, int IN, int OUT>
int launch_gemv(const GemvArgs& p, const void* x, const void* z, const void* w, void* out, void* h_out, hipStream_t stream) {
  constexpr bool GLU = OUT == OUT_GLU || OUT == OUT_ROUTER_GLU;
  const int F = GLU ? (p.N - p.routers) / 2 : p.N;
  const size_t lds = (size_t)p.M * p.K * (p.M == 1 ? 4 : sizeof(T));
  auto go = [&](auto r_tag, auto m_tag) -> int {
    constexpr int R = decltype(r_tag)::value, MR = decltype(m_tag)::value;
    constexpr int OR = GLU ? R / 2 : R;
    auto* k = gemv_kernel<T, IN, OUT, R, MR>;
    if (lds > 64 * 1024) {
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    const int units = (p.routers + R - 1) / R + (F + OR - 1) / OR;
    k<<<dim3((unsigned)((units + 3) / 4)), 256, lds, stream>>>(p, (const T*)x, (const T*)z, (const T*)w, (T*)out, (T*)h_out);
    return launched();
  };
  auto rows = [&](auto m_tag) -> int {
    // two rows per wavefront once that still leaves four wavefronts per SIMD (four rows were slower: 13.6 against 10.1 us
    // for 8704 x 2048, 29.7 against 26.9 us for 16896 x 4096)
    if (GLU || F >= 4096) return go(std::integral_constant<int, 2>{}, m_tag);
    return go(std::integral_constant<int, GLU ? 2 : 1>{}, m_tag);
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

extern "C" int aqs_gemv(int in_kind, int out_kind, int dtype, const void* x, int64_t ldx, const float* xf, const float* yf,
                        const float* post, float* x_out, const float* gain, float gain0, float eps, int64_t groups, const void* w,
                        const float* bias, float mult, float limit, int64_t routers, float* res, void* out, int64_t ldo, void* h_out,
                        int64_t M, int64_t N, int64_t K, void* stream) {
  SQ_CHECK(M >= 0 && N > 0 && K > 0, AQ_E_SHAPE);
  if (M == 0) return AQ_OK;
  SQ_CHECK(aqs_gemv_ok(dtype, M, N, K), AQ_E_SHAPE);
  const bool glu = out_kind >= OUT_GLU;
  SQ_NEED(w && (out_kind == OUT_F32 || out_kind == OUT_RESIDUAL ? (const void*)res : (const void*)out));
  SQ_CHECK(!bad_ptr16(w) && (in_kind == IN_GATED_NORM || !bad_ptr16(x)) && !bad_ptr16(xf) && !bad_ptr16(gain) && !bad_ptr16(yf) &&
               !bad_ptr16(post) && !bad_ptr16(x_out), AQ_E_ALIGN);
  SQ_CHECK(out_kind == OUT_ROUTER_GLU ? routers > 0 && routers < N : routers == 0, AQ_E_SHAPE);
  SQ_CHECK(!glu || (N - routers) % 2 == 0, AQ_E_SHAPE);
  SQ_CHECK(ldo >= (glu ? (N - routers) / 2 : N), AQ_E_SHAPE);
  GemvArgs p{};
  p.xf = xf, p.yf = yf, p.post = post, p.x_out = x_out, p.gain = gain, p.gain0 = gain0, p.bias = bias, p.res = res, p.ldo = ldo;
  p.M = (int)M, p.N = (int)N, p.K = (int)K, p.groups = (int)groups, p.routers = (int)routers;
  p.eps = eps, p.mult = mult, p.limit = limit;
  const void* z = nullptr;
  if (in_kind == IN_PLAIN || in_kind == IN_ROW_NORM) {
    SQ_NEED(x && (in_kind == IN_PLAIN || gain));
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
    } else if (in_kind == IN_NORM_GATE) {
      SQ_NEED(x);
      SQ_CHECK(ldx >= K && ldx % 8 == 0, AQ_E_SHAPE);
      z = x, p.ldz = ldx;
    } else if (in_kind == IN_POST_RMSNORM) {
      SQ_NEED(yf && post && x_out);
      SQ_CHECK(x_out != xf, AQ_E_SHAPE);  // other workgroups still read the old stream
    }
  }
  SQ_NEED(out_kind != OUT_ROUTER_GLU || (res && h_out));
  hipStream_t st = (hipStream_t)stream;
#define SQ_GEMV(I, O) \
  if (in_kind == I && out_kind == O) SQ_DISPATCH(dtype, return (launch_gemv<T, I, O>(p, x, z, w, out, h_out, st)))
  SQ_GEMV(IN_PLAIN, OUT_T);
  SQ_GEMV(IN_PLAIN, OUT_F32);
  SQ_GEMV(IN_PLAIN, OUT_RESIDUAL);
  SQ_GEMV(IN_RMSNORM, OUT_T);
  SQ_GEMV(IN_RMSNORM, OUT_F32);
  SQ_GEMV(IN_RMSNORM, OUT_GLU);
  SQ_GEMV(IN_GATED_NORM, OUT_RESIDUAL);
  SQ_GEMV(IN_POST_RMSNORM, OUT_T);
  SQ_GEMV(IN_POST_RMSNORM, OUT_F32);
  SQ_GEMV(IN_POST_RMSNORM, OUT_ROUTER_GLU);
  SQ_GEMV(IN_ROW_NORM, OUT_T);
  SQ_GEMV(IN_NORM_GATE, OUT_F32);
#undef SQ_GEMV
  return AQ_E_SHAPE;
}
