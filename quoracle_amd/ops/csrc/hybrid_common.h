// Element access shared by the kernels that run in bf16 and in float32.
#pragma once

#include "common.h"

namespace hyb {

__device__ __forceinline__ float to_f(float v) { return v; }
__device__ __forceinline__ float to_f(bf16 v) { return bf2f(v); }
__device__ __forceinline__ void put(float *p, float v) { *p = v; }
__device__ __forceinline__ void put(bf16 *p, float v) { *p = f2bf(v); }

// VEC (1 or 4) consecutive elements as floats; 4 needs natural alignment of
// the whole group.
template <int VEC>
__device__ __forceinline__ void load_v(const float *p, float *o) {
  if constexpr (VEC == 4) {
    const float4 v = *reinterpret_cast<const float4 *>(p);
    o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
  } else {
    o[0] = *p;
  }
}
template <int VEC>
__device__ __forceinline__ void load_v(const bf16 *p, float *o) {
  if constexpr (VEC == 4) {
    const uint2 v = *reinterpret_cast<const uint2 *>(p);
    unpack_bf16x2(v.x, o[0], o[1]);
    unpack_bf16x2(v.y, o[2], o[3]);
  } else {
    o[0] = bf2f(*p);
  }
}
template <int VEC>
__device__ __forceinline__ void store_v(float *p, const float *v) {
  if constexpr (VEC == 4)
    *reinterpret_cast<float4 *>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else
    *p = v[0];
}
template <int VEC>
__device__ __forceinline__ void store_v(bf16 *p, const float *v) {
  if constexpr (VEC == 4)
    *reinterpret_cast<uint2 *>(p) =
        make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
  else
    *p = f2bf(v[0]);
}

__device__ __forceinline__ float sigmoid_f(float z) {
  return 1.f / (1.f + expf(-z));
}

// Gate/activation selectors used by several kernels.
enum Act : int { ACT_NONE = 0, ACT_SILU = 1, ACT_SIGMOID = 2 };

__device__ __forceinline__ float activate(float z, int act) {
  if (act == ACT_SILU) return z * sigmoid_f(z);
  if (act == ACT_SIGMOID) return sigmoid_f(z);
  return z;
}

}  // namespace hyb
