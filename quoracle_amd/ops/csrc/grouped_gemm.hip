// Grouped matrix products C = A B^T on one launch (gfx950): the products of a
// mixture of experts, where each group has its own rows, and those of latent
// attention, where a group is a head and every group has the same rows.
//
//   B [groups][N][K] row-major, so both operands are contiguous along K.
//   bf16 with K, the strides and the group offsets multiples of 8: MFMA
//     gg_tile_kernel    tiles copied straight into LDS (many rows)
//     gg_strip_kernel   16 rows x 32 columns per wave, operands straight from
//                       memory; the waves share the columns' K range (weights
//                       are read once, decode) or take columns side by side
//   anything else, and float32: gg_plain_kernel.
//
// Rows.  Without a tile list blockIdx.z is the group and it has M rows.  With
// one, a workgroup takes a tile of it: group, first row and number of rows, 0
// for tiles that are not there; tile_count says how many are.  `rows` maps a row of the sorted order to a slot
// (token * top + k): A's row is then slot / a_div (a_div > 0) or the row
// itself, C's row the slot (c_slot) or the row itself, and scale[slot]
// multiplies the product before the gelu.
#pragma once

#include "hybrid_common.h"

typedef __bf16 gg_b16x8 __attribute__((ext_vector_type(8)));
typedef float gg_f32x4 __attribute__((ext_vector_type(4)));
typedef float gg_f32x16 __attribute__((ext_vector_type(16)));

struct GroupedGemm {
  const void *a, *b;
  void *c;
  long lda, ldc;
  long a_group, c_group;               // element offset of a group's columns
  int M, N, K;
  const int *tile_group, *tile_row0, *tile_rows, *tile_count;
  int row_tiles;                       // tiles of the list, or of a group
  const int *rows;
  int a_div;
  bool c_slot;
  const float *scale;
  bool gelu;
};

namespace gg {

struct Tile {
  int group, row0, rows;
};

__device__ __forceinline__ Tile tile_of(const GroupedGemm &p, int BM, int i) {
  if (p.tile_group)
    return {p.tile_group[i], p.tile_row0[i], p.tile_rows[i]};
  const int row0 = i * BM;
  return {(int)blockIdx.z, row0, min(BM, p.M - row0)};
}

__device__ __forceinline__ long a_row(const GroupedGemm &p, int row) {
  return p.rows && p.a_div ? p.rows[row] / p.a_div : row;
}

// What becomes of row `row`: where it goes and its scale.
struct Out {
  long at;
  float scale;
};

__device__ __forceinline__ Out out_row(const GroupedGemm &p, const Tile &t,
                                       int row) {
  const int slot = p.rows ? p.rows[row] : row;
  return {(p.c_slot ? slot : row) * p.ldc + t.group * p.c_group,
          p.scale ? p.scale[slot] : 1.f};
}

template <typename T>
__device__ __forceinline__ float finish(const GroupedGemm &p, float v,
                                        float scale) {
  v *= scale;
  return p.gelu ? hyb::gelu<T>(v) : v;
}

}  // namespace gg

// 16 bytes of zeros, copied where a row ends before a step does.
__device__ const uint4 gg_zeros = {0, 0, 0, 0};

// ---------------------------------------------------------------------------
// BM x BN tile, 64 deep, two buffers in LDS; WM x WN waves.  Rows of 64 values
// in LDS hold their vector v at v ^ swizzle(row), so that the rows of a column
// do not meet in a bank.  Each die takes a run of neighbouring tiles, four row
// tiles before the next columns: they share an expert's rows and weights.
// Grid: (ceil(N/BN) * tiles, 1, groups); block 64 * WM * WN.
// ---------------------------------------------------------------------------
template <int BM, int BN, int WM, int WN>
__global__ void __launch_bounds__(64 * WM * WN, 2)
gg_tile_kernel(GroupedGemm p) {
  constexpr int BK = 64, NW = WM * WN, G = 4;
  constexpr int MI = BM / WM / 32, NJ = BN / WN / 32;
  constexpr int IA = BM / 8 / NW, IB = BN / 8 / NW;   // copies of 8 rows
  __shared__ __align__(16) bf16 a_s[2][BM * BK];
  __shared__ __align__(16) bf16 b_s[2][BN * BK];
  const int cols = (p.N + BN - 1) / BN;
  const int n_rows = p.tile_count ? *p.tile_count : p.row_tiles;
  const int total = n_rows * cols;
  int at = blockIdx.x;
  if (at >= total) return;
  {
    const int die = at % 8, rest = total % 8;
    at = die * (total / 8) + min(die, rest) + at / 8;
  }
  const int band = at / (G * cols), in = at % (G * cols);
  const int high = min(G, n_rows - band * G);
  const gg::Tile tile = gg::tile_of(p, BM, band * G + in % high);
  if (tile.rows <= 0) return;
  const int n0 = in / high * BN;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int wm = wave / WN, wn = wave % WN;
  const int l31 = lane & 31, half = lane >> 5;
  const bf16 *a = (const bf16 *)p.a + tile.group * p.a_group;
  const bf16 *b = (const bf16 *)p.b + (long)tile.group * p.N * p.K;

  // copy i of this wave: rows 8 * (wave + i * NW) + lane / 8 (the last one
  // again behind it), at kv of a step
  static_assert(NW % 2 == 0, "rows of a copy keep their swizzle");
  const int lr = lane >> 3;
  const int kv = ((lane & 7) ^ ((wave * 8 + lr) >> 1 & 7)) * 8;
  const bf16 *ap[IA], *bp[IB];
#pragma unroll
  for (int i = 0; i < IA; ++i) {
    const int r = min((wave + i * NW) * 8 + lr, tile.rows - 1);
    ap[i] = a + gg::a_row(p, tile.row0 + r) * p.lda + kv;
  }
#pragma unroll
  for (int i = 0; i < IB; ++i) {
    const int r = min(n0 + (wave + i * NW) * 8 + lr, p.N - 1);
    bp[i] = b + (long)r * p.K + kv;
  }
  auto fetch = [&](int k0, int buf) {
    const bool there = k0 + kv < p.K;
#pragma unroll
    for (int i = 0; i < IA; ++i)
      hyb::dma16(there ? (const void *)(ap[i] + k0) : &gg_zeros,
                 &a_s[buf][(wave + i * NW) * 512]);
#pragma unroll
    for (int i = 0; i < IB; ++i)
      hyb::dma16(there ? (const void *)(bp[i] + k0) : &gg_zeros,
                 &b_s[buf][(wave + i * NW) * 512]);
  };
  gg_f32x16 acc[MI][NJ];
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < NJ; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.f;

  fetch(0, 0);
  const int sw = l31 >> 1 & 7;
  for (int k0 = 0, buf = 0; k0 < p.K; k0 += BK, buf ^= 1) {
    // also: the other buffer's readers are done
    hyb::dma_barrier();
    if (k0 + BK < p.K) fetch(k0 + BK, buf ^ 1);
    const bf16 *as = &a_s[buf][(wm * (BM / WM) + l31) * BK];
    const bf16 *bs = &b_s[buf][(wn * (BN / WN) + l31) * BK];
#pragma unroll
    for (int kk = 0; kk < BK / 16; ++kk) {
      const int v = ((kk * 2 + half) ^ sw) * 8;
      gg_b16x8 af[MI], bfr[NJ];
#pragma unroll
      for (int i = 0; i < MI; ++i)
        af[i] = *reinterpret_cast<const gg_b16x8 *>(as + i * 32 * BK + v);
#pragma unroll
      for (int j = 0; j < NJ; ++j)
        bfr[j] = *reinterpret_cast<const gg_b16x8 *>(bs + j * 32 * BK + v);
#pragma unroll
      for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < NJ; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
              af[i], bfr[j], acc[i][j], 0, 0, 0);
    }
  }
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int row = wm * (BM / WM) + i * 32 + (r & 3) + 8 * (r >> 2) +
                      4 * half;
      if (row >= tile.rows) continue;
      const gg::Out o = gg::out_row(p, tile, tile.row0 + row);
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        const int col = n0 + wn * (BN / WN) + j * 32 + l31;
        if (col < p.N)
          ((bf16 *)p.c)[o.at + col] =
              f2bf(gg::finish<bf16>(p, acc[i][j][r], o.scale));
      }
    }
}

// ---------------------------------------------------------------------------
// 16 rows.  SPLIT: the four waves take every fourth 32-deep step of the same
// 32 columns and join their sums in LDS; otherwise each wave takes 32 columns
// of its own.  Grid: (ceil(N / (SPLIT ? 32 : 128)), tiles, groups); block 256.
// ---------------------------------------------------------------------------
template <bool SPLIT>
__global__ void __launch_bounds__(256) gg_strip_kernel(GroupedGemm p) {
  const gg::Tile tile = gg::tile_of(p, 16, blockIdx.y);
  if (tile.rows <= 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int l15 = lane & 15, g = lane >> 4;
  const int n0 = SPLIT ? blockIdx.x * 32 : blockIdx.x * 128 + wave * 32;
  const bf16 *a = (const bf16 *)p.a + tile.group * p.a_group;
  const bf16 *b = (const bf16 *)p.b + (long)tile.group * p.N * p.K;
  const bool a_ok = l15 < tile.rows;
  const bf16 *ap =
      a_ok ? a + gg::a_row(p, tile.row0 + l15) * p.lda + g * 8 : a;
  const bool b_ok[2] = {n0 + l15 < p.N, n0 + 16 + l15 < p.N};
  const bf16 *bp[2];
#pragma unroll
  for (int j = 0; j < 2; ++j)
    bp[j] = b + (b_ok[j] ? (long)(n0 + 16 * j + l15) * p.K + g * 8 : 0);

  gg_f32x4 acc[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
  constexpr int STEP = SPLIT ? 128 : 32, U = 4;
  for (int k0 = SPLIT ? wave * 32 : 0; k0 < p.K; k0 += STEP * U) {
    uint4 av[U], bv[U][2];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * STEP;
      const bool in = k + g * 8 < p.K;
      av[u] = in && a_ok ? *reinterpret_cast<const uint4 *>(ap + k)
                         : make_uint4(0, 0, 0, 0);
#pragma unroll
      for (int j = 0; j < 2; ++j)
        bv[u][j] = in && b_ok[j] ? *reinterpret_cast<const uint4 *>(bp[j] + k)
                                 : make_uint4(0, 0, 0, 0);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int j = 0; j < 2; ++j)
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            __builtin_bit_cast(gg_b16x8, av[u]),
            __builtin_bit_cast(gg_b16x8, bv[u][j]), acc[j], 0, 0, 0);
  }
  if constexpr (SPLIT) {
    __shared__ float part[4][16][33];
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        part[wave][g * 4 + r][j * 16 + l15] = acc[j][r];
    __syncthreads();
    for (int i = threadIdx.x; i < 16 * 32; i += 256) {
      const int row = i / 32, col = i % 32;
      if (row >= tile.rows || n0 + col >= p.N) continue;
      const float v = part[0][row][col] + part[1][row][col] +
                      part[2][row][col] + part[3][row][col];
      const gg::Out o = gg::out_row(p, tile, tile.row0 + row);
      ((bf16 *)p.c)[o.at + n0 + col] = f2bf(gg::finish<bf16>(p, v, o.scale));
    }
  } else {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = g * 4 + r;
      if (row >= tile.rows) continue;
      const gg::Out o = gg::out_row(p, tile, tile.row0 + row);
#pragma unroll
      for (int j = 0; j < 2; ++j)
        if (b_ok[j])
          ((bf16 *)p.c)[o.at + n0 + 16 * j + l15] =
              f2bf(gg::finish<bf16>(p, acc[j][r], o.scale));
    }
  }
}

// ---------------------------------------------------------------------------
// Any sizes, any alignment: 16 x 64 tiles on the vector ALU.
// Grid: (ceil(N/64), tiles, groups); block 256.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(256) gg_plain_kernel(GroupedGemm p) {
  constexpr int BK = 32;
  __shared__ float a_s[16][BK + 1];
  __shared__ float b_s[64][BK + 1];
  const gg::Tile tile = gg::tile_of(p, 16, blockIdx.y);
  if (tile.rows <= 0) return;
  const int n0 = blockIdx.x * 64, tid = threadIdx.x;
  const int col = tid & 63, r0 = tid >> 6;
  const T *a = (const T *)p.a + tile.group * p.a_group;
  const T *b = (const T *)p.b + (long)tile.group * p.N * p.K;
  float acc[4] = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < p.K; k0 += BK) {
    for (int i = tid; i < 16 * BK; i += 256) {
      const int r = i / BK, k = k0 + i % BK;
      a_s[r][i % BK] =
          r < tile.rows && k < p.K
              ? hyb::to_f(a[gg::a_row(p, tile.row0 + r) * p.lda + k])
              : 0.f;
    }
    for (int i = tid; i < 64 * BK; i += 256) {
      const int r = i / BK, k = k0 + i % BK;
      b_s[r][i % BK] = n0 + r < p.N && k < p.K
                           ? hyb::to_f(b[(long)(n0 + r) * p.K + k])
                           : 0.f;
    }
    __syncthreads();
    for (int k = 0; k < BK; ++k) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        acc[i] = fmaf(a_s[r0 + 4 * i][k], b_s[col][k], acc[i]);
    }
    __syncthreads();
  }
  if (n0 + col >= p.N) return;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = r0 + 4 * i;
    if (row >= tile.rows) continue;
    const gg::Out o = gg::out_row(p, tile, tile.row0 + row);
    hyb::put((T *)p.c + o.at + n0 + col,
             gg::finish<T>(p, acc[i], o.scale));
  }
}
