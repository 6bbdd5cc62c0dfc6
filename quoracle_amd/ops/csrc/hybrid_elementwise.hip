// Elementwise, norm and gate kernels of the recurrent and chunk-local mixers.  T is the activation type (bf16 or float); the residual stream, all
// norms, gates of a recurrence and position angles are float32.
//
// VEC > 1 kernels need every row start to be a multiple of VEC elements.
// Norm kernels keep their row in registers: NI groups of VEC per thread.
// NI = 0 (rows that do not fit) reads the row a second time instead.

#include "hybrid_common.h"

// ---------------------------------------------------------------------------
// Norm after the sum: x <- rms(alpha*x + sa*a (+ sb*b)) * w in place;
// h = T(x).  Grid: (T); block 256.
// ---------------------------------------------------------------------------
template <typename T, int VEC, int NI>
__global__ void __launch_bounds__(256)
post_norm_kernel(float *__restrict__ x, T *__restrict__ h,
                 const T *__restrict__ a, float sa, const T *__restrict__ b,
                 float sb, float alpha, const float *__restrict__ w, int n,
                 float eps) {
  __shared__ float scratch[4];
  const long row = (long)blockIdx.x * n;
  auto sum_at = [&](int i, float *xv) {
    float av[VEC];
    hyb::load_v<VEC>(x + row + i, xv);
    hyb::load_v<VEC>(a + row + i, av);
#pragma unroll
    for (int k = 0; k < VEC; ++k) xv[k] = alpha * xv[k] + sa * av[k];
    if (b) {
      hyb::load_v<VEC>(b + row + i, av);
#pragma unroll
      for (int k = 0; k < VEC; ++k) xv[k] += sb * av[k];
    }
  };
  auto finish = [&](int i, float *xv, float inv) {
    float wv[VEC];
    hyb::load_v<VEC>(w + i, wv);
#pragma unroll
    for (int k = 0; k < VEC; ++k) xv[k] = xv[k] * inv * wv[k];
    hyb::store_v<VEC>(x + row + i, xv);
    hyb::store_v<VEC>(h + row + i, xv);
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
      for (int k = 0; k < VEC; ++k) ssq += v[it][k] * v[it][k];
    }
    const float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int i = (it * 256 + threadIdx.x) * VEC;
      if (i < n) finish(i, v[it], inv);
    }
  } else {
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
      float v[VEC];
      sum_at(i, v);
#pragma unroll
      for (int k = 0; k < VEC; ++k) ssq += v[k] * v[k];
    }
    const float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
      float v[VEC];
      sum_at(i, v);
      finish(i, v, inv);
    }
  }
}

// ---------------------------------------------------------------------------
// out = silu(gu[:, :n]) * gu[:, n:].  Grid: (T, ceil(n / (256*VEC))).
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
glu_kernel(T *__restrict__ out, const T *__restrict__ gu, int n) {
  const long t = blockIdx.x;
  const int i = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (i >= n) return;
  float g[VEC], u[VEC];
  hyb::load_v<VEC>(gu + t * 2 * n + i, g);
  hyb::load_v<VEC>(gu + t * 2 * n + n + i, u);
#pragma unroll
  for (int k = 0; k < VEC; ++k) g[k] = g[k] * hyb::sigmoid_t<T>(g[k]) * u[k];
  hyb::store_v<VEC>(out + t * n + i, g);
}

// ---------------------------------------------------------------------------
// Norm each group of `n` values of o[t] (a head, or all heads together),
// times w[n], times act(gate): out[t, g*n + i].  The gate is read in place
// from the fused projection row.  Grid: (T, groups); block 256.
// ---------------------------------------------------------------------------
template <typename T, int VEC, int NI>
__global__ void __launch_bounds__(256)
gated_norm_kernel(T *__restrict__ out, const T *__restrict__ o,
                  const T *__restrict__ proj, long stride, int g_off,
                  const float *__restrict__ w, int n, int act, float eps) {
  __shared__ float scratch[4];
  const long t = blockIdx.x;
  const long base = (t * gridDim.y + blockIdx.y) * (long)n;
  const T *gate = proj + t * stride + g_off + (long)blockIdx.y * n;
  auto finish = [&](int i, float *v, const float *gv, float inv) {
    float wv[VEC];
    hyb::load_v<VEC>(w + i, wv);
#pragma unroll
    for (int k = 0; k < VEC; ++k)
      v[k] = v[k] * inv * wv[k] * hyb::activate<T>(gv[k], act);
    hyb::store_v<VEC>(out + base + i, v);
  };
  float ssq = 0.f;
  if constexpr (NI > 0) {
    float v[NI][VEC], gv[NI][VEC];       // the gate is on its way meanwhile
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int i = (it * 256 + threadIdx.x) * VEC;
      if (i >= n) continue;
      hyb::load_v<VEC>(o + base + i, v[it]);
      hyb::load_v<VEC>(gate + i, gv[it]);
#pragma unroll
      for (int k = 0; k < VEC; ++k) ssq += v[it][k] * v[it][k];
    }
    const float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
#pragma unroll
    for (int it = 0; it < NI; ++it) {
      const int i = (it * 256 + threadIdx.x) * VEC;
      if (i < n) finish(i, v[it], gv[it], inv);
    }
  } else {
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
      float v[VEC];
      hyb::load_v<VEC>(o + base + i, v);
#pragma unroll
      for (int k = 0; k < VEC; ++k) ssq += v[k] * v[k];
    }
    const float inv = 1.f / sqrtf(block_sum(ssq, scratch) / (float)n + eps);
    for (int i = threadIdx.x * VEC; i < n; i += 256 * VEC) {
      float v[VEC], gv[VEC];
      hyb::load_v<VEC>(o + base + i, v);
      hyb::load_v<VEC>(gate + i, gv);
      finish(i, v, gv, inv);
    }
  }
}

// The same for groups of at most LPG*VEC values: LPG lanes per group, many
// groups per workgroup.  Grid: ceil(T*groups*LPG / 256); block 256.
template <typename T, int VEC, int LPG>
__global__ void __launch_bounds__(256)
gated_norm_small_kernel(T *__restrict__ out, const T *__restrict__ o,
                        const T *__restrict__ proj, long stride, int g_off,
                        const float *__restrict__ w, int n, int groups,
                        long total, int act, float eps) {
  const long at = ((long)blockIdx.x * 256 + threadIdx.x) / LPG;
  const int i = (threadIdx.x % LPG) * VEC;
  const bool live = at < total && i < n;
  float v[VEC], gv[VEC], wv[VEC];
  float ssq = 0.f;
  if (live) {
    hyb::load_v<VEC>(o + at * n + i, v);
    hyb::load_v<VEC>(
        proj + at / groups * stride + g_off + at % groups * n + i, gv);
    hyb::load_v<VEC>(w + i, wv);
#pragma unroll
    for (int k = 0; k < VEC; ++k) ssq += v[k] * v[k];
  }
#pragma unroll
  for (int s = LPG / 2; s >= 1; s >>= 1) ssq += __shfl_xor(ssq, s, LPG);
  if (!live) return;
  const float inv = 1.f / sqrtf(ssq / (float)n + eps);
#pragma unroll
  for (int k = 0; k < VEC; ++k)
    v[k] = v[k] * inv * wv[k] * hyb::activate<T>(gv[k], act);
  hyb::store_v<VEC>(out + at * n + i, v);
}

// ---------------------------------------------------------------------------
// Attention input of one token, fused: RMS norm over the whole query and over
// the whole key projection, rotation of the interleaved pairs (2i, 2i+1) of
// the first 2*n_pairs dimensions of each head by pos * freq[i] (cos and sin
// times `mag`), queries out, rotated keys and the raw projected keys (the
// values) into the paged cache.
// Grid: (T); block 256; dynamic LDS 2*n_pairs floats.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256)
qk_norm_rope_store_kernel(
    T *__restrict__ q_out, T *__restrict__ kcache, T *__restrict__ vcache,
    const T *__restrict__ proj, long stride, int q_off, int k_off,
    const float *__restrict__ qw, const float *__restrict__ kw,
    const int *__restrict__ positions, const int *__restrict__ slots,
    const double *__restrict__ freq, int n_pairs, float mag, float eps, int H,
    int G, int D, int BS) {
  extern __shared__ float rot_s[];
  __shared__ float scratch[4];
  float *cos_s = rot_s, *sin_s = rot_s + n_pairs;
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const T *qp = proj + t * stride + q_off;
  const T *kp = proj + t * stride + k_off;
  const int nq = H * D, nk = G * D;
  const double pos = (double)positions[t];
  for (int i = tid; i < n_pairs; i += 256) {
    // whole turns taken off before the angle becomes a float
    double turns = pos * freq[i] * 0.15915494309189535;
    turns -= rint(turns);
    float s, c;
    sincosf((float)(turns * 6.283185307179586), &s, &c);
    cos_s[i] = c * mag;
    sin_s[i] = s * mag;
  }
  float sq = 0.f, sk = 0.f;
  for (int i = tid; i < nq; i += 256) {
    const float v = hyb::to_f(qp[i]);
    sq += v * v;
  }
  for (int i = tid; i < nk; i += 256) {
    const float v = hyb::to_f(kp[i]);
    sk += v * v;
  }
  const float qi = 1.f / sqrtf(block_sum(sq, scratch) / (float)nq + eps);
  const float ki = 1.f / sqrtf(block_sum(sk, scratch) / (float)nk + eps);

  const int slot = slots[t];
  const long blk = slot / BS;
  const int off = slot % BS;
  const int hp = (D + 1) / 2;                    // pairs per head
  for (int p = tid; p < (H + G) * hp; p += 256) {
    const int head = p / hp, pr = p % hp;
    const bool is_q = head < H;
    const int i0 = (is_q ? head : head - H) * D + 2 * pr;
    const bool two = 2 * pr + 1 < D;
    const T *src = is_q ? qp : kp;
    const float *w = is_q ? qw : kw;
    const float inv = is_q ? qi : ki;
    const float r0 = hyb::to_f(src[i0]);
    const float r1 = two ? hyb::to_f(src[i0 + 1]) : 0.f;
    float u = r0 * inv * w[i0];
    float v = two ? r1 * inv * w[i0 + 1] : 0.f;
    if (pr < n_pairs) {
      const float c = cos_s[pr], s = sin_s[pr];
      const float a = u * c - v * s;
      v = v * c + u * s;
      u = a;
    }
    if (is_q) {
      T *dst = q_out + t * nq + i0;
      hyb::put(dst, u);
      if (two) hyb::put(dst + 1, v);
    } else if (slot >= 0) {
      const long at =
          ((blk * G + (head - H)) * (long)BS + off) * D + 2 * pr;
      hyb::put(kcache + at, u);
      hyb::put(vcache + at, r0);
      if (two) {
        hyb::put(kcache + at + 1, v);
        hyb::put(vcache + at + 1, r1);
      }
    }
  }
}

// The same for head dimensions, offsets and rows that are multiples of 8:
// eight elements (four pairs) at a time, the token's groups held in
// registers.  NI groups per thread.
template <typename T, int NI>
__global__ void __launch_bounds__(256)
qk_norm_rope_store8_kernel(
    T *__restrict__ q_out, T *__restrict__ kcache, T *__restrict__ vcache,
    const T *__restrict__ proj, long stride, int q_off, int k_off,
    const float *__restrict__ qw, const float *__restrict__ kw,
    const int *__restrict__ positions, const int *__restrict__ slots,
    const double *__restrict__ freq, int n_pairs, float mag, float eps, int H,
    int G, int D, int BS) {
  extern __shared__ float rot_s[];
  __shared__ float scratch[8];
  float *cos_s = rot_s, *sin_s = rot_s + n_pairs;
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const T *row = proj + t * stride;
  const int nq = H * D, nk = G * D, n8 = (nq + nk) / 8;
  float x[NI][8];
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int it = 0; it < NI; ++it) {
    const int i = (it * 256 + tid) * 8;
    if (i >= n8 * 8) continue;
    hyb::load_v<8>(row + (i < nq ? q_off + i : k_off + i - nq), x[it]);
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < 8; ++k) s += x[it][k] * x[it][k];
    if (i < nq) sq += s;
    else sk += s;
  }
  const double pos = (double)positions[t];
  for (int i = tid; i < n_pairs; i += 256) {
    double turns = pos * freq[i] * 0.15915494309189535;
    turns -= rint(turns);
    float s, c;
    sincosf((float)(turns * 6.283185307179586), &s, &c);
    cos_s[i] = c * mag;
    sin_s[i] = s * mag;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((tid & 63) == 0) {
    scratch[tid >> 6] = sq;
    scratch[4 + (tid >> 6)] = sk;
  }
  __syncthreads();                     // also publishes cos_s / sin_s
  sq = scratch[0] + scratch[1] + scratch[2] + scratch[3];
  sk = scratch[4] + scratch[5] + scratch[6] + scratch[7];
  const float qi = 1.f / sqrtf(sq / (float)nq + eps);
  const float ki = 1.f / sqrtf(sk / (float)nk + eps);
  const int slot = slots[t];
  const long blk = slot / BS;
  const int off = slot % BS;
#pragma unroll
  for (int it = 0; it < NI; ++it) {
    const int i = (it * 256 + tid) * 8;
    if (i >= n8 * 8) continue;
    const bool is_q = i < nq;
    const int at = is_q ? i : i - nq;
    const int head = at / D, d = at % D;
    const float inv = is_q ? qi : ki;
    float w[8], y[8];
    hyb::load_v<8>((is_q ? qw : kw) + at, w);
#pragma unroll
    for (int k = 0; k < 8; ++k) y[k] = x[it][k] * inv * w[k];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int pr = d / 2 + k;
      if (pr < n_pairs) {
        const float c = cos_s[pr], s = sin_s[pr];
        const float u = y[2 * k], v = y[2 * k + 1];
        y[2 * k] = u * c - v * s;
        y[2 * k + 1] = v * c + u * s;
      }
    }
    if (is_q) {
      hyb::store_v<8>(q_out + t * nq + at, y);
    } else if (slot >= 0) {
      const long dst = ((blk * G + head) * (long)BS + off) * D + d;
      hyb::store_v<8>(kcache + dst, y);
      hyb::store_v<8>(vcache + dst, x[it]);
    }
  }
}

// ---------------------------------------------------------------------------
// Log of a low-rank sigmoid decay per key channel, summed along runs of
// consecutive rows:
//   z = A2 a1[t] + b,  ld[t] = log(sigmoid(z)) / tau,
//   out[t] = ld[t] + out[t-1] inside a run (the first row of a run: ld[t]).
// run_row0 null: every row is a run of its own (out = ld).
// A workgroup takes 64 channels; its four waves take 16 rows each of every 64
// and join their sums.  RMAX: rank the channel's weights are held in
// registers for; 0: any rank.
// Grid: (runs, ceil(C/64)); block 256.
// ---------------------------------------------------------------------------
// log(sigmoid(z)) = min(z, 0) - log(1 + e), e = exp(-|z|).  For bf16 models
// with the hardware exponential and logarithm, and the series of log(1 + e)
// where 1 + e would round away e (both within 2^-20 of the value).
template <typename T> __device__ __forceinline__ float log_sigmoid(float z) {
  if constexpr (sizeof(T) == 2) {
    const float e = __expf(-fabsf(z));
    const float series =
        e * (1.f - e * (0.5f - e * (0.33333333f - e * (0.25f - e * 0.2f))));
    return fminf(z, 0.f) - (e < 0.0625f ? series : __logf(1.f + e));
  } else {
    return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
  }
}

template <typename T, int RMAX>
__global__ void __launch_bounds__(256)
log_decay_kernel(float *__restrict__ out, const T *__restrict__ proj,
                 long stride, int a_off, int rank, const T *__restrict__ a2,
                 const float *__restrict__ bias, float inv_tau, int C,
                 const int *__restrict__ run_row0,
                 const int *__restrict__ run_len) {
  constexpr int TB = 64;
  constexpr int RS = RMAX ? RMAX : 1;
  __shared__ __align__(16) float a_s[TB * RS];
  __shared__ float sum_s[4][64];
  const int lane = threadIdx.x & 63;
  const int quarter = threadIdx.x >> 6;
  const int c = min((int)blockIdx.y * 64 + lane, C - 1);
  const bool live = (int)blockIdx.y * 64 + lane < C;
  const long row0 = run_row0 ? run_row0[blockIdx.x] : (int)blockIdx.x;
  const int len = run_row0 ? run_len[blockIdx.x] : 1;
  const T *wr = a2 + (long)c * rank;
  const float b = bias[c];
  float w[RS];
  if (RMAX > 0 && quarter * 16 < len) {
    if (rank == RMAX) {
#pragma unroll
      for (int r = 0; r < RS / 8; ++r) hyb::load_v<8>(wr + 8 * r, w + 8 * r);
    } else {
#pragma unroll
      for (int r = 0; r < RS; ++r) w[r] = r < rank ? hyb::to_f(wr[r]) : 0.f;
    }
  }
  float carry = 0.f;
  for (int t0 = 0; t0 < len; t0 += TB) {
    const int tn = min(TB, len - t0);
    const T *a = proj + (row0 + t0) * stride + a_off;
    if constexpr (RMAX > 0) {
      for (int i = threadIdx.x; i < tn * RMAX; i += 256) {
        const int t = i / RMAX, r = i % RMAX;
        a_s[i] = r < rank ? hyb::to_f(a[t * stride + r]) : 0.f;
      }
      __syncthreads();
    }
    float part[16], sum = 0.f;
#pragma unroll
    for (int u = 0; u < 16; ++u) {
      const int t = quarter * 16 + u;
      if (t < tn) {                                   // wave-uniform
        float z = b;
        if constexpr (RMAX > 0) {
#pragma unroll
          for (int r = 0; r < RMAX; ++r) z = fmaf(w[r], a_s[t * RMAX + r], z);
        } else {
          for (int r = 0; r < rank; ++r)
            z = fmaf(hyb::to_f(wr[r]), hyb::to_f(a[t * stride + r]), z);
        }
        sum += log_sigmoid<T>(z) * inv_tau;
      }
      part[u] = sum;
    }
    sum_s[quarter][lane] = sum;
    __syncthreads();
    float before = carry;
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      if (q < quarter) before += sum_s[q][lane];
      carry += sum_s[q][lane];
    }
#pragma unroll
    for (int u = 0; u < 16; ++u) {
      const int t = quarter * 16 + u;
      if (t < tn && live) out[(row0 + t0 + t) * (long)C + c] = before + part[u];
    }
    if (t0 + TB < len) __syncthreads();
  }
}
