// Norms, rotation and activation around latent attention and feed-forwards.  T
// is the activation type (bf16 or float); the residual stream, all norms and
// position angles are float32 (angles are reduced in double).
//
// VEC > 1 kernels need every row start to be a multiple of VEC elements.

#include "hybrid_common.h"

// ---------------------------------------------------------------------------
// Residual sum of a normed sublayer output, and the norm that follows:
//   s = sum over K terms of y[t] (+ bias) (+ gate[t] * y2[t])
//   x += rms(s) * w
//   joined[t, :n] = T(x) if given (rows of 2n);  h = T(rms(x) * w_next) if
//   w_next is given.
// NI groups of VEC per thread are held in registers; NI = 0 (rows that do not
// fit) keeps them in x instead.  Grid: (T); block 256.
// ---------------------------------------------------------------------------
template <typename T, int VEC, int NI>
__global__ void __launch_bounds__(256)
sandwich_norm_kernel(float *__restrict__ x, T *__restrict__ h,
                     T *__restrict__ joined, const float *__restrict__ w_next,
                     const T *__restrict__ y, int K,
                     const float *__restrict__ bias, const T *__restrict__ y2,
                     const float *__restrict__ gate,
                     const float *__restrict__ w, int n, float eps) {
  __shared__ float scratch[4];
  const long t = blockIdx.x;
  const long row = t * n;
  const float g = gate ? gate[t] : 0.f;
  auto sum_at = [&](int i, float *v) {
    hyb::load_v<VEC>(y + row * K + i, v);
    float a[VEC];
    for (int k = 1; k < K; ++k) {
      hyb::load_v<VEC>(y + row * K + (long)k * n + i, a);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += a[j];
    }
    if (bias) {
      hyb::load_v<VEC>(bias + i, a);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] += a[j];
    }
    if (y2) {
      hyb::load_v<VEC>(y2 + row + i, a);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = fmaf(g, a[j], v[j]);
    }
  };
  // x at i becomes x + v * inv * w, in v
  auto add_at = [&](int i, float *v, float inv) {
    float xv[VEC], wv[VEC];
    hyb::load_v<VEC>(x + row + i, xv);
    hyb::load_v<VEC>(w + i, wv);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] = fmaf(v[j] * inv, wv[j], xv[j]);
    hyb::store_v<VEC>(x + row + i, v);
    if (joined) hyb::store_v<VEC>(joined + 2 * row + i, v);
  };
  auto norm_at = [&](int i, const float *v, float inv) {
    float o[VEC];
    hyb::load_v<VEC>(w_next + i, o);
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] *= v[j] * inv;
    hyb::store_v<VEC>(h + row + i, o);
  };
  float ssq = 0.f;
  if constexpr (NI > 0) {
    float v[NI][VEC];
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int i = (it * 256 + threadIdx.x) * VEC;
      if (i >= n) continue;
      sum_at(i, v[it]);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ssq += v[it][j] * v[it][j];
    }
    float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
    ssq = 0.f;
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int i = (it * 256 + threadIdx.x) * VEC;
      if (i >= n) continue;
      add_at(i, v[it], inv);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ssq += v[it][j] * v[it][j];
    }
    if (!w_next) return;
    inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int i = (it * 256 + threadIdx.x) * VEC;
      if (i < n) norm_at(i, v[it], inv);
    }
  } else {
    float v[VEC];
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
      sum_at(i, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ssq += v[j] * v[j];
    }
    float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
    ssq = 0.f;
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
      sum_at(i, v);
      add_at(i, v, inv);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ssq += v[j] * v[j];
    }
    if (!w_next) return;
    inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
      hyb::load_v<VEC>(x + row + i, v);     // this thread's own stores
      norm_at(i, v, inv);
    }
  }
}

// cos and sin of pos * freq[i] into LDS, whole turns taken off in double.
__device__ __forceinline__ void fill_angles(float *cos_s, float *sin_s,
                                            int pos, const double *freq,
                                            int n_pairs) {
  for (int i = threadIdx.x; i < n_pairs; i += blockDim.x) {
    double turns = (double)pos * freq[i] * 0.15915494309189535;
    turns -= rint(turns);
    float s, c;
    sincosf((float)(turns * 6.283185307179586), &s, &c);
    cos_s[i] = c;
    sin_s[i] = s;
  }
}

// ---------------------------------------------------------------------------
// One token's latents, from its row of the fused projection: the query latent
// (q_rank values at 0) normed with wq into cq; the key/value latent (rank
// values at kv_off) normed with wkv and the rotated key part behind it
// (2 * n_pairs values) into the token's slot of the paged pool, at 0 and at
// rank_p.  Grid: (T); block 256; dynamic LDS 2 * n_pairs floats.
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
latent_store_kernel(T *__restrict__ cq, T *__restrict__ pool,
                    const T *__restrict__ proj, long stride, int q_rank,
                    int kv_off, int rank, int rank_p, int width,
                    const float *__restrict__ wq,
                    const float *__restrict__ wkv,
                    const int *__restrict__ positions,
                    const int *__restrict__ slots,
                    const double *__restrict__ freq, int n_pairs, float eps) {
  extern __shared__ float rot_s[];
  __shared__ float scratch[8];
  float *cos_s = rot_s, *sin_s = rot_s + n_pairs;
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const T *qp = proj + t * stride;
  const T *kp = qp + kv_off;
  const int slot = slots[t];
  float sq = 0.f, sk = 0.f, v[VEC], wv[VEC];
  // both parts as one list of groups, queries first
  for (int i = tid * VEC; i < q_rank + rank; i += 256 * VEC) {
    const bool is_q = i < q_rank;
    hyb::load_v<VEC>(is_q ? qp + i : kp + i - q_rank, v);
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < VEC; ++j) s += v[j] * v[j];
    if (is_q) sq += s;
    else sk += s;
  }
  fill_angles(cos_s, sin_s, positions[t], freq, n_pairs);
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((tid & 63) == 0) {
    scratch[tid >> 6] = sq;
    scratch[4 + (tid >> 6)] = sk;
  }
  __syncthreads();                       // also publishes the angles
  sq = scratch[0] + scratch[1] + scratch[2] + scratch[3];
  sk = scratch[4] + scratch[5] + scratch[6] + scratch[7];
  const float qi = 1.f / sqrtf(sq / (float)q_rank + eps);
  const float ki = 1.f / sqrtf(sk / (float)rank + eps);
  T *dst = pool + (long)slot * width;
  for (int i = tid * VEC; i < q_rank + rank; i += 256 * VEC) {
    const bool is_q = i < q_rank;
    const int at = is_q ? i : i - q_rank;
    hyb::load_v<VEC>(is_q ? qp + at : kp + at, v);
    hyb::load_v<VEC>((is_q ? wq : wkv) + at, wv);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] = v[j] * (is_q ? qi : ki) * wv[j];
    if (is_q) hyb::store_v<VEC>(cq + t * q_rank + at, v);
    else if (slot >= 0) hyb::store_v<VEC>(dst + at, v);
  }
  if (slot < 0) return;
  for (int p = tid; p < n_pairs; p += 256) {
    const float a = hyb::to_f(kp[rank + 2 * p]);
    const float b = hyb::to_f(kp[rank + 2 * p + 1]);
    hyb::put(dst + rank_p + 2 * p, a * cos_s[p] - b * sin_s[p]);
    hyb::put(dst + rank_p + 2 * p + 1, b * cos_s[p] + a * sin_s[p]);
  }
}

// ---------------------------------------------------------------------------
// Rotate the interleaved pairs of columns off .. off + 2*n_pairs of every head
// of q [T, H, D] in place, PV pairs at a time.
// Grid: (T); block 256; dynamic LDS 2 * n_pairs floats.
// ---------------------------------------------------------------------------
template <typename T, int PV>
__global__ void __launch_bounds__(256)
rotate_heads_kernel(T *__restrict__ q, int H, int D, int off,
                    const int *__restrict__ positions,
                    const double *__restrict__ freq, int n_pairs) {
  extern __shared__ float rot_s[];
  float *cos_s = rot_s, *sin_s = rot_s + n_pairs;
  const long t = blockIdx.x;
  fill_angles(cos_s, sin_s, positions[t], freq, n_pairs);
  __syncthreads();
  const int groups = n_pairs / PV;
  for (int i = threadIdx.x; i < H * groups; i += 256) {
    const int head = i / groups, p0 = i % groups * PV;
    T *at = q + (t * H + head) * D + off + 2 * p0;
    float v[2 * PV];
    if constexpr (PV == 4) {
      hyb::load_v<8>(at, v);
    } else {
      v[0] = hyb::to_f(at[0]);
      v[1] = hyb::to_f(at[1]);
    }
#pragma unroll
    for (int k = 0; k < PV; ++k) {
      const float c = cos_s[p0 + k], s = sin_s[p0 + k];
      const float a = v[2 * k], b = v[2 * k + 1];
      v[2 * k] = a * c - b * s;
      v[2 * k + 1] = b * c + a * s;
    }
    if constexpr (PV == 4) {
      hyb::store_v<8>(at, v);
    } else {
      hyb::put(at, v[0]);
      hyb::put(at + 1, v[1]);
    }
  }
}

// ---------------------------------------------------------------------------
// z = gelu(z + bias) in place, the exact form.
// Grid: (T, ceil(n / (256*VEC))); block 256.
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
bias_gelu_kernel(T *__restrict__ z, const float *__restrict__ bias, int n) {
  const int i = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (i >= n) return;
  T *at = z + (long)blockIdx.x * n + i;
  float v[VEC];
  hyb::load_v<VEC>(at, v);
  if (bias) {
    float b[VEC];
    hyb::load_v<VEC>(bias + i, b);
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[k] += b[k];
  }
#pragma unroll
  for (int k = 0; k < VEC; ++k) v[k] = hyb::gelu<T>(v[k]);
  hyb::store_v<VEC>(at, v);
}
