// Router of a mixture of experts and the order of rows its products run in
// (gfx950).  The products themselves are in grouped_gemm.hip.

#include "grouped_gemm.hip"

// One wave picks the `top` largest of s[0..E): repeated maxima, the lower
// index first among equals.  s is LDS that this wave owns; it is consumed
// (volatile: the lanes read what lane 0 wrote).
__device__ __forceinline__ void pick_top(volatile float *s, int E, int top,
                                         int *__restrict__ ids,
                                         float *__restrict__ weights) {
  const int lane = threadIdx.x & 63;
  for (int k = 0; k < top; ++k) {
    float best = -1.f;                       // below every sigmoid
    int at = E;
    for (int e = lane; e < E; e += 64) {
      const float v = s[e];
      if (v > best) { best = v; at = e; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float b2 = __shfl_xor(best, o, 64);
      const int a2 = __shfl_xor(at, o, 64);
      if (b2 > best || (b2 == best && a2 < at)) { best = b2; at = a2; }
    }
    if (at >= E) at = 0;                     // scores that are not numbers
    if (lane == 0) {
      ids[k] = at;
      weights[k] = best;
      s[at] = -1.f;
    }
    __builtin_amdgcn_wave_barrier();
  }
}

// ---------------------------------------------------------------------------
// Scores sigmoid(router h) of E experts (and of one more row, the gate, when
// `gate` is given), the `top` largest with their scores.  One token per
// workgroup.  Grid: (T); block 256; dynamic LDS E floats.
// ---------------------------------------------------------------------------
template <typename T, int VEC>
__global__ void __launch_bounds__(256)
moe_route_kernel(int *__restrict__ ids, float *__restrict__ weights,
                 float *__restrict__ gate, const T *__restrict__ h,
                 const T *__restrict__ router, int n, int E, int top) {
  extern __shared__ float score_s[];
  const long t = blockIdx.x;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  for (int e = wave; e < E + (gate != nullptr); e += 4) {
    float dot = 0.f, a[VEC], w[VEC];
    for (int i = lane * VEC; i < n; i += 64 * VEC) {
      hyb::load_v<VEC>(h + t * n + i, a);
      hyb::load_v<VEC>(router + (long)e * n + i, w);
#pragma unroll
      for (int k = 0; k < VEC; ++k) dot = fmaf(a[k], w[k], dot);
    }
    const float s = hyb::sigmoid_f(wave_sum(dot));
    if (lane == 0) {
      if (e < E) score_s[e] = s;
      else gate[t] = s;
    }
  }
  __syncthreads();
  if (wave == 0)
    pick_top(score_s, E, top, ids + t * top, weights + t * top);
}

// The same for 16 tokens per workgroup on the matrix cores (bf16 products are
// exact in float32): eight waves take every eighth 32-deep step, 64 columns at
// a time.  Grid: (ceil(T/16)); block 512; dynamic LDS 16 * (E + 1) floats.
__global__ void __launch_bounds__(512)
moe_route_mfma_kernel(int *__restrict__ ids, float *__restrict__ weights,
                      float *__restrict__ gate, const bf16 *__restrict__ h,
                      const bf16 *__restrict__ router, int T, int n, int E,
                      int top) {
  extern __shared__ float score_s[];
  __shared__ float part[8][16][65];
  const int t0 = blockIdx.x * 16;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int l15 = lane & 15, g = lane >> 4;
  const int cols = E + (gate != nullptr);
  const bool a_ok = t0 + l15 < T;
  const bf16 *ap = h + (a_ok ? (long)(t0 + l15) * n : 0) + g * 8;
  for (int c0 = 0; c0 < cols; c0 += 64) {
    gg_f32x4 acc[4];
    const bf16 *bp[4];
    bool b_ok[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      acc[j] = (gg_f32x4){0.f, 0.f, 0.f, 0.f};
      b_ok[j] = c0 + 16 * j + l15 < cols;
      bp[j] = router + (b_ok[j] ? (long)(c0 + 16 * j + l15) * n : 0) + g * 8;
    }
    constexpr int U = 4;                     // steps under way
    for (int k0 = wave * 32; k0 < n; k0 += 256 * U) {
      uint4 av[U], bv[U][4];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = k0 + u * 256;
        const bool in = k + g * 8 < n;
        av[u] = in && a_ok ? *reinterpret_cast<const uint4 *>(ap + k)
                           : make_uint4(0, 0, 0, 0);
#pragma unroll
        for (int j = 0; j < 4; ++j)
          bv[u][j] = in && b_ok[j]
                         ? *reinterpret_cast<const uint4 *>(bp[j] + k)
                         : make_uint4(0, 0, 0, 0);
      }
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c0 + 16 * j < cols)
            acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                __builtin_bit_cast(gg_b16x8, av[u]),
                __builtin_bit_cast(gg_b16x8, bv[u][j]), acc[j], 0, 0, 0);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        part[wave][g * 4 + r][16 * j + l15] = acc[j][r];
    __syncthreads();
    for (int i = threadIdx.x; i < 16 * 64; i += 512) {
      const int row = i / 64, e = c0 + i % 64;
      if (e >= cols) continue;
      float z = 0.f;
#pragma unroll
      for (int w = 0; w < 8; ++w) z += part[w][row][i % 64];
      const float s = hyb::sigmoid_f(z);
      if (e < E) score_s[row * (E + 1) + e] = s;
      else if (t0 + row < T) gate[t0 + row] = s;
    }
    __syncthreads();
  }
  for (int row = wave; row < 16; row += 8)
    if (t0 + row < T)
      pick_top(score_s + row * (E + 1), E, top, ids + (long)(t0 + row) * top,
               weights + (long)(t0 + row) * top);
}

// ---------------------------------------------------------------------------
// Slots (token * top + k) in the order of their experts, and the list of row
// tiles (BM rows of one expert each) and its length; unused tiles get 0 rows.
// Grid: (1); block 1024; dynamic LDS 3 * E ints.
// ---------------------------------------------------------------------------
__global__ void __launch_bounds__(1024)
moe_order_kernel(int *__restrict__ rows, int *__restrict__ tile_group,
                 int *__restrict__ tile_row0, int *__restrict__ tile_rows,
                 int *__restrict__ tile_count,
                 const int *__restrict__ ids, int S, int E, int BM,
                 int n_tiles) {
  extern __shared__ int order_s[];
  int *count = order_s, *first = order_s + E, *tile0 = order_s + 2 * E;
  __shared__ int used;
  for (int e = threadIdx.x; e < E; e += 1024) count[e] = 0;
  __syncthreads();
  for (int i = threadIdx.x; i < S; i += 1024) atomicAdd(&count[ids[i]], 1);
  __syncthreads();
  if (threadIdx.x < 64) {                    // exclusive sums, one wave
    int at = 0, tl = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + threadIdx.x;
      const int c = e < E ? count[e] : 0, nt = (c + BM - 1) / BM;
      int cs = c, ts = nt;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int c2 = __shfl_up(cs, o, 64), t2 = __shfl_up(ts, o, 64);
        if ((int)threadIdx.x >= o) { cs += c2; ts += t2; }
      }
      if (e < E) {
        first[e] = at + cs - c;
        tile0[e] = tl + ts - nt;
      }
      at += __shfl(cs, 63, 64);
      tl += __shfl(ts, 63, 64);
    }
    if (threadIdx.x == 0) *tile_count = used = tl;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += 1024)
    for (int j = 0, t = tile0[e]; j < count[e]; j += BM, ++t) {
      tile_group[t] = e;
      tile_row0[t] = first[e] + j;
      tile_rows[t] = min(BM, count[e] - j);
    }
  for (int t = used + threadIdx.x; t < n_tiles; t += 1024) {
    tile_group[t] = 0;
    tile_row0[t] = 0;
    tile_rows[t] = 0;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < S; i += 1024)
    rows[atomicAdd(&first[ids[i]], 1)] = i;
}
