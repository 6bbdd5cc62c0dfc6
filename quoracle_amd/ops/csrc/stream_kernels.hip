// Kernels of the float32 residual stream that all hybrid models share.  T is
// the activation type (bf16 or float).
//
// VEC > 1 kernels need every row start to be a multiple of VEC elements.

#include "hybrid_common.h"

// ---------------------------------------------------------------------------
// x[t] = embed[tokens[t]] (+ table[positions[t]]); h = T(x).
// Grid: (T); block 256.
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
embed_positions_kernel(float *__restrict__ x, T *__restrict__ h,
                       const T *__restrict__ embed,
                       const T *__restrict__ table,
                       const int *__restrict__ tokens,
                       const int *__restrict__ positions, int n) {
  const long t = blockIdx.x;
  const T *e = embed + (long)tokens[t] * n;
  const T *p = table ? table + (long)positions[t] * n : nullptr;
  for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
    float a[VEC], b[VEC];
    hyb::load_v<VEC>(e + i, a);
    if (p) {
      hyb::load_v<VEC>(p + i, b);
#pragma unroll
      for (int k = 0; k < VEC; ++k) a[k] += b[k];
    }
    hyb::store_v<VEC>(x + t * n + i, a);
    hyb::store_v<VEC>(h + t * n + i, a);
  }
}

// ---------------------------------------------------------------------------
// out[r] = T(rms(x[rows[r]]) * w): the final norm of the rows that need
// logits.  Grid: (R); block 256.
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
norm_rows_kernel(T *__restrict__ out, const float *__restrict__ x,
                 const long *__restrict__ rows, const float *__restrict__ w,
                 int n, float eps) {
  __shared__ float scratch[4];
  const float *src = x + rows[blockIdx.x] * (long)n;
  T *dst = out + (long)blockIdx.x * n;
  float ssq = 0.f;
  for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
    float v[VEC];
    hyb::load_v<VEC>(src + i, v);
#pragma unroll
    for (int k = 0; k < VEC; ++k) ssq += v[k] * v[k];
  }
  const float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
  for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
    float v[VEC], wv[VEC];
    hyb::load_v<VEC>(src + i, v);
    hyb::load_v<VEC>(w + i, wv);
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[k] = v[k] * inv * wv[k];
    hyb::store_v<VEC>(dst + i, v);
  }
}

// ---------------------------------------------------------------------------
// x[t] = y[t] if y is given; h[t] = T(rms(x[t]) * w).  Grid: (T); block 256.
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
pre_norm_kernel(float *__restrict__ x, T *__restrict__ h,
                const float *__restrict__ y, const float *__restrict__ w,
                int n, float eps) {
  __shared__ float scratch[4];
  const long row = (long)blockIdx.x * n;
  const float *src = (y ? y : x) + row;
  float ssq = 0.f;
  for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
    float v[VEC];
    hyb::load_v<VEC>(src + i, v);
#pragma unroll
    for (int k = 0; k < VEC; ++k) ssq += v[k] * v[k];
  }
  const float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
  for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
    float v[VEC], wv[VEC];
    hyb::load_v<VEC>(src + i, v);
    hyb::load_v<VEC>(w + i, wv);
    if (y) hyb::store_v<VEC>(x + row + i, v);
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[k] = v[k] * inv * wv[k];
    hyb::store_v<VEC>(h + row + i, v);
  }
}
