// Grouped matrix products C = A B^T on one launch (gfx950): the products of a
// mixture of experts, where each group has its own rows, and those of latent
// attention, where a group is a head and every group has the same rows.
//
//   B [groups][N][K] row-major, so both operands are contiguous along K.
//   bf16 with K, the strides and the group offsets multiples of 8: MFMA
//     gg_tile_kernel    BM x 128 tiles staged through LDS (many rows)
//     gg_strip_kernel   16 rows x 32 columns per wave, operands straight from
//                       memory; the waves share the columns' K range (weights
//                       are read once, decode) or take columns side by side
//   anything else, and float32: gg_plain_kernel.
//
// Rows.  Without a tile list blockIdx.z is the group and it has M rows.  With
// one, blockIdx.y is a tile: group, first row and number of rows, 0 for tiles
// that are not there.  `rows` maps a row of the sorted order to a slot
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
  const int *tile_group, *tile_row0, *tile_rows;
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

__device__ __forceinline__ Tile tile_of(const GroupedGemm &p, int BM) {
  if (p.tile_group) {
    const int i = blockIdx.y;
    return {p.tile_group[i], p.tile_row0[i], p.tile_rows[i]};
  }
  const int row0 = blockIdx.y * BM;
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

// ---------------------------------------------------------------------------
// BM x 128 tile, 64 deep, double-buffered in LDS; four waves of (BM/2) x 64.
// Grid: (ceil(N/128), tiles, groups); block 256.
// ---------------------------------------------------------------------------
template <int BM>
__global__ void __launch_bounds__(256, 2) gg_tile_kernel(GroupedGemm p) {
  constexpr int BN = 128, BK = 64, LS = BK + 8;
  constexpr int NA = BM * BK / 8 / 256, NBV = BN * BK / 8 / 256;
  constexpr int MI = BM / 64;                  // 32-row blocks of a wave
  __shared__ __align__(16) bf16 a_s[2][BM * LS];
  __shared__ __align__(16) bf16 b_s[2][BN * LS];
  const gg::Tile tile = gg::tile_of(p, BM);
  if (tile.rows <= 0) return;
  const int n0 = blockIdx.x * BN;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int wm = wave >> 1, wn = wave & 1;
  const int l31 = lane & 31, half = lane >> 5;
  const bf16 *a = (const bf16 *)p.a + tile.group * p.a_group;
  const bf16 *b = (const bf16 *)p.b + (long)tile.group * p.N * p.K;

  const bf16 *a_at[NA], *b_at[NBV];            // null: rows that are not there
#pragma unroll
  for (int i = 0; i < NA; ++i) {
    const int r = (tid + i * 256) / (BK / 8);
    a_at[i] = r < tile.rows
                  ? a + gg::a_row(p, tile.row0 + r) * p.lda + tid % 8 * 8
                  : nullptr;
  }
#pragma unroll
  for (int i = 0; i < NBV; ++i) {
    const int r = (tid + i * 256) / (BK / 8);
    b_at[i] = n0 + r < p.N ? b + (long)(n0 + r) * p.K + tid % 8 * 8 : nullptr;
  }
  uint4 ar[NA], br[NBV];
  auto load = [&](int k0) {
    const bool in = k0 + tid % 8 * 8 < p.K;
#pragma unroll
    for (int i = 0; i < NA; ++i)
      ar[i] = in && a_at[i] ? *reinterpret_cast<const uint4 *>(a_at[i] + k0)
                            : make_uint4(0, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < NBV; ++i)
      br[i] = in && b_at[i] ? *reinterpret_cast<const uint4 *>(b_at[i] + k0)
                            : make_uint4(0, 0, 0, 0);
  };
  auto stage = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NA; ++i) {
      const int j = tid + i * 256;
      *reinterpret_cast<uint4 *>(&a_s[buf][j / 8 * LS + j % 8 * 8]) = ar[i];
    }
#pragma unroll
    for (int i = 0; i < NBV; ++i) {
      const int j = tid + i * 256;
      *reinterpret_cast<uint4 *>(&b_s[buf][j / 8 * LS + j % 8 * 8]) = br[i];
    }
  };
  gg_f32x16 acc[MI][2];
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.f;

  load(0);
  stage(0);
  __syncthreads();
  for (int k0 = 0, buf = 0; k0 < p.K; k0 += BK, buf ^= 1) {
    const bool more = k0 + BK < p.K;
    if (more) load(k0 + BK);
#pragma unroll
    for (int kk = 0; kk < BK / 16; ++kk) {
      gg_b16x8 af[MI], bfr[2];
#pragma unroll
      for (int i = 0; i < MI; ++i)
        af[i] = *reinterpret_cast<const gg_b16x8 *>(
            &a_s[buf][(wm * (BM / 2) + i * 32 + l31) * LS + kk * 16 +
                      half * 8]);
#pragma unroll
      for (int j = 0; j < 2; ++j)
        bfr[j] = *reinterpret_cast<const gg_b16x8 *>(
            &b_s[buf][(wn * 64 + j * 32 + l31) * LS + kk * 16 + half * 8]);
#pragma unroll
      for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
              af[i], bfr[j], acc[i][j], 0, 0, 0);
    }
    // the other buffer: its readers passed the barrier of the last step
    if (more) stage(buf ^ 1);
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int row = wm * (BM / 2) + i * 32 + (r & 3) + 8 * (r >> 2) +
                      4 * half;
      if (row >= tile.rows) continue;
      const gg::Out o = gg::out_row(p, tile, tile.row0 + row);
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int col = n0 + wn * 64 + j * 32 + l31;
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
  const gg::Tile tile = gg::tile_of(p, 16);
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
  const gg::Tile tile = gg::tile_of(p, 16);
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
