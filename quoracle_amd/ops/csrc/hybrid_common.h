// Element access shared by the kernels that run in bf16 and in float32.
#pragma once

#include "common.h"

namespace hyb {

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16 v) { return bf2f(v); }
__device__ __forceinline__ void put(float *p, float v) { *p = v; }
__device__ __forceinline__ void put(bf16 *p, float v) { *p = f2bf(v); }

// VEC (1, 4 or 8) consecutive elements as floats; 4 and 8 need the whole
// group at its natural alignment (at most 16 bytes).
template <int VEC>
__device__ __forceinline__ void load_v(const float *p, float *o) {
  if constexpr (VEC == 1) {
    o[0] = *p;
  } else {
#pragma unroll
    for (int i = 0; i < VEC / 4; ++i) {
      const float4 v = reinterpret_cast<const float4 *>(p)[i];
      o[4 * i] = v.x; o[4 * i + 1] = v.y;
      o[4 * i + 2] = v.z; o[4 * i + 3] = v.w;
    }
  }
}
template <int VEC>
__device__ __forceinline__ void load_v(const bf16 *p, float *o) {
  if constexpr (VEC == 1) {
    o[0] = bf2f(*p);
  } else if constexpr (VEC == 4) {
    const uint2 v = *reinterpret_cast<const uint2 *>(p);
    unpack_bf16x2(v.x, o[0], o[1]);
    unpack_bf16x2(v.y, o[2], o[3]);
  } else {
    const uint4 v = *reinterpret_cast<const uint4 *>(p);
    unpack_bf16x2(v.x, o[0], o[1]);
    unpack_bf16x2(v.y, o[2], o[3]);
    unpack_bf16x2(v.z, o[4], o[5]);
    unpack_bf16x2(v.w, o[6], o[7]);
  }
}
template <int VEC>
__device__ __forceinline__ void store_v(float *p, const float *v) {
  if constexpr (VEC == 1) {
    *p = v[0];
  } else {
#pragma unroll
    for (int i = 0; i < VEC / 4; ++i)
      reinterpret_cast<float4 *>(p)[i] =
          make_float4(v[4 * i], v[4 * i + 1], v[4 * i + 2], v[4 * i + 3]);
  }
}
template <int VEC>
__device__ __forceinline__ void store_v(bf16 *p, const float *v) {
  if constexpr (VEC == 1)
    *p = f2bf(v[0]);
  else if constexpr (VEC == 4)
    *reinterpret_cast<uint2 *>(p) =
        make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
  else
    *reinterpret_cast<uint4 *>(p) =
        make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]),
                   pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
}

__device__ __forceinline__ float sigmoid_f(float z) {
  return 1.f / (1.f + expf(-z));
}

// The sigmoid of an activation or gate that is rounded to T afterwards: for
// bf16 the hardware exponential and reciprocal, good to a few 2^-22.
template <typename T> __device__ __forceinline__ float sigmoid_t(float z) {
  if constexpr (sizeof(T) == 2)
    return __builtin_amdgcn_rcpf(1.f + __expf(-z));
  else
    return sigmoid_f(z);
}

// Gate/activation selectors used by several kernels.
enum Act : int { ACT_NONE = 0, ACT_SILU = 1, ACT_SIGMOID = 2 };

template <typename T>
__device__ __forceinline__ float activate(float z, int act) {
  if (act == ACT_SILU) return z * sigmoid_t<T>(z);
  if (act == ACT_SIGMOID) return sigmoid_t<T>(z);
  return z;
}

// z * Phi(z), the exact (erf) gelu.  For values that are rounded to bf16
// afterwards erf(|u|) = 1 - P(t) exp(-u^2), t = 1 / (1 + 0.3275911 |u|), with
// P of degree five: Abramowitz and Stegun, Handbook of Mathematical Functions,
// 7.1.26, absolute error below 1.5e-7.
template <typename T> __device__ __forceinline__ float gelu(float z) {
  const float u = z * 0.70710678f;
  if constexpr (sizeof(T) == 2) {
    const float t = __builtin_amdgcn_rcpf(fmaf(0.3275911f, fabsf(u), 1.f));
    float p = fmaf(1.061405429f, t, -1.453152027f);
    p = fmaf(p, t, 1.421413741f);
    p = fmaf(p, t, -0.284496736f);
    p = fmaf(p, t, 0.254829592f);
    const float e = 1.f - p * t * __expf(-u * u);
    return 0.5f * z * (1.f + copysignf(e, u));
  } else {
    return 0.5f * z * (1.f + erff(u));
  }
}

// Copy 16 bytes per lane from memory straight into LDS: lane i's go to
// `to` + 16 i, lanes that are switched off leave their place as it is.  The
// copy is under way until the wave's vector-memory counter says otherwise, see
// dma_barrier().  (The wait state is what a write of M0 needs before its use.)
__device__ __forceinline__ void dma16(const void *from, void *to) {
  const unsigned at = __builtin_amdgcn_readfirstlane(
      (unsigned)(size_t)(__attribute__((address_space(3))) void *)to);
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\t"
               "global_load_lds_dwordx4 %1, off"
               :
               : "s"(at), "v"(from)
               : "memory", "m0");
}
// Barrier behind which every wave's copies so far are in LDS.
__device__ __forceinline__ void dma_barrier() {
  asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");
}
// Barrier for LDS only: copies stay under way.
__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

}  // namespace hyb
