// Shared device helpers of the hybrid-sequence kernels (convolutions, linear recurrences, windowed
// attention, the row operations and matrix-vector products around them).  Activations and weights
// are bf16 or fp32 (template parameter T); everything between a load and a store is fp32.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include <type_traits>

#include "../../include/astrai_q.h"
#include "../../include/astrai_seq.h"

namespace sq {

struct bf16 {
  uint16_t bits;
};

__device__ __forceinline__ float to_f32(float v) { return v; }
__device__ __forceinline__ float to_f32(bf16 v) { return __uint_as_float((uint32_t)v.bits << 16); }

__device__ __forceinline__ uint32_t pack2(float lo, float hi) {
  typedef float f2 __attribute__((ext_vector_type(2)));
  typedef __bf16 b2 __attribute__((ext_vector_type(2)));
  const f2 v = {lo, hi};
  return __builtin_bit_cast(uint32_t, __builtin_convertvector(v, b2));
}
template <typename T>
__device__ __forceinline__ T from_f32(float v);
template <>
__device__ __forceinline__ float from_f32<float>(float v) {
  return v;
}
template <>
__device__ __forceinline__ bf16 from_f32<bf16>(float v) {
  return bf16{(uint16_t)(pack2(v, v) & 0xffffu)};
}

// N consecutive elements (N * sizeof(T) a multiple of 8 bytes, p aligned to it or to 16) as fp32
template <int N>
__device__ __forceinline__ void load_vec(const float* p, float (&o)[N]) {
  static_assert(N % 2 == 0, "pairs");
  if constexpr (N % 4 == 0) {
#pragma unroll
    for (int i = 0; i < N / 4; ++i) {
      const float4 v = reinterpret_cast<const float4*>(p)[i];
      o[4 * i] = v.x, o[4 * i + 1] = v.y, o[4 * i + 2] = v.z, o[4 * i + 3] = v.w;
    }
  } else {
#pragma unroll
    for (int i = 0; i < N / 2; ++i) {
      const float2 v = reinterpret_cast<const float2*>(p)[i];
      o[2 * i] = v.x, o[2 * i + 1] = v.y;
    }
  }
}
__device__ __forceinline__ void unpack8(uint4 v, float* o) {
  const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    o[2 * i] = __uint_as_float(w[i] << 16);
    o[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
  }
}
// eight elements of T, 16-byte aligned, kept as they are until they are used
template <typename T>
struct Raw8;
template <>
struct Raw8<bf16> {
  uint4 v;
  __device__ __forceinline__ void load(const bf16* p) { v = *reinterpret_cast<const uint4*>(p); }
  __device__ __forceinline__ void zero() { v = make_uint4(0, 0, 0, 0); }
  __device__ __forceinline__ void get(float* o) const { unpack8(v, o); }
};
template <>
struct Raw8<float> {
  float4 a, b;
  __device__ __forceinline__ void load(const float* p) {
    a = reinterpret_cast<const float4*>(p)[0];
    b = reinterpret_cast<const float4*>(p)[1];
  }
  __device__ __forceinline__ void zero() { a = b = make_float4(0, 0, 0, 0); }
  __device__ __forceinline__ void get(float* o) const {
    o[0] = a.x, o[1] = a.y, o[2] = a.z, o[3] = a.w, o[4] = b.x, o[5] = b.y, o[6] = b.z, o[7] = b.w;
  }
};

// ---- cross-lane sums
#define SQ_DPP_ADD(v, ctrl) \
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), ctrl, 0xf, 0xf, true))
// over each row of 16 consecutive lanes, in all of them
__device__ __forceinline__ float row16_sum(float v) {
  SQ_DPP_ADD(v, 0xB1);   // quad_perm [1,0,3,2]
  SQ_DPP_ADD(v, 0x4E);   // quad_perm [2,3,0,1]
  SQ_DPP_ADD(v, 0x141);  // row_half_mirror
  SQ_DPP_ADD(v, 0x140);  // row_mirror
  return v;
}
__device__ __forceinline__ float wave_sum(float v) {
  v = row16_sum(v);
  v += __shfl_xor(v, 16, 64);
  v += __shfl_xor(v, 32, 64);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = 32; o; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}
// Sum over a workgroup of WAVES wavefronts, in every thread.  red: WAVES floats of LDS; two barriers.
template <int WAVES>
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.0f;
#pragma unroll
  for (int i = 0; i < WAVES; ++i) s += red[i];
  return s;
}

// ---- elementwise functions (fp32)
// e^x and 1 / (1 + e^-x) from the hardware's exp2 and reciprocal (each within an ulp or two)
__device__ __forceinline__ float exp_fast(float x) { return __builtin_amdgcn_exp2f(x * 1.44269504088896341f); }
__device__ __forceinline__ float sigmoid(float x) { return __builtin_amdgcn_rcpf(1.0f + exp_fast(-x)); }
__device__ __forceinline__ float silu(float x) { return x * sigmoid(x); }
// log(1 + exp(x)) without overflow, to full relative precision
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.0f) + log1pf(expf(-fabsf(x))); }
// the same within 1e-7 absolutely: enough where only exp(-a softplus) is used
__device__ __forceinline__ float softplus_abs(float x) {
  return fmaxf(x, 0.0f) + 0.693147180559945309f * __builtin_amdgcn_logf(1.0f + exp_fast(-fabsf(x)));
}
// g * sigmoid(1.702 g) * (u + 1) of the clamped pair: the gate from above only, the linear part on both sides
__device__ __forceinline__ float clamped_glu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid(1.702f * g) * (u + 1.0f);
}

inline int bad_ptr16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15u) != 0; }
inline int launched() { return (int)hipGetLastError(); }

}  // namespace sq

#define SQ_NEED(p)                  \
  do {                              \
    if (!(p)) return AQ_E_NULL;     \
  } while (0)
#define SQ_CHECK(cond, code)        \
  do {                              \
    if (!(cond)) return (code);     \
  } while (0)
// the statement behind the dtype names the element type T
#define SQ_DISPATCH(dtype, ...)                  \
  do {                                           \
    if ((dtype) == AQ_BF16) {                    \
      using T = sq::bf16;                        \
      __VA_ARGS__;                               \
    } else if ((dtype) == AQ_F32) {              \
      using T = float;                           \
      __VA_ARGS__;                               \
    } else {                                     \
      return AQ_E_DTYPE;                         \
    }                                            \
  } while (0)
