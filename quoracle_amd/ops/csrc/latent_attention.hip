// Attention over paged latents (gfx950).  A cached token is one row of the
// pool [num_blocks, BS, rank + rot]: a latent of `rank` values from which
// every head's key and value are made, and one rotated key part of `rot`
// values for all heads.  Both widths are padded to multiples of 8 with zeros.
//
//   latent space   The key part of the query is taken into the latent space
//                  (one small product per head), so that all heads attend to
//                  the cached rows themselves and the values are the same
//                  latents: decoding and short portions (latent_tile_kernel,
//                  bf16; latent_rows_kernel, any size and float32).
//   expanded       Keys and values of the whole context are made first by a
//                  plain product: long portions (expanded_prefill_kernel).
//
// Softmax with a sink: the running softmax of a row starts from a key of score
// sink[head] that has no value (m = sink, l = 1) instead of from nothing.
// Scores and softmax are float32; the weights enter the matrix cores as a bf16
// pair (hi + lo), so that they keep 16 significant bits.
#pragma once

#include "hybrid_common.h"

typedef __bf16 la_b16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 la_b16x8 __attribute__((ext_vector_type(8)));
typedef short la_s16x4 __attribute__((ext_vector_type(4)));
typedef float la_f32x4 __attribute__((ext_vector_type(4)));
typedef float la_f32x16 __attribute__((ext_vector_type(16)));

namespace la {

// Transposed LDS read of a 4 x 16 block of 16-bit values by 16 lanes: lane i
// points at row i/4, columns i%4*4 and gets column i of the four rows.
__device__ __forceinline__ la_b16x4 read_tr(const bf16 *at) {
  typedef __attribute__((address_space(3))) la_s16x4 lds_s16x4;
  const la_s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (lds_s16x4 *)const_cast<bf16 *>(at));
  return __builtin_bit_cast(la_b16x4, v);
}

__device__ __forceinline__ la_b16x8 join4(la_b16x4 a, la_b16x4 b) {
  return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
}

// Join NS partial softmaxes: weight of part i and their sum.  The parts lie
// `step` apart from base.  All threads of a 128-thread block take part.
__device__ __forceinline__ float part_max(const float *part_m, long base,
                                          long step, int NS, float *scratch) {
  float m = -INFINITY;
  for (int i = threadIdx.x; i < NS; i += blockDim.x)
    m = fmaxf(m, part_m[base + i * step]);
  return block_max(m, scratch);
}

}  // namespace la

// ---------------------------------------------------------------------------
// Latent space.  Query rows are the flattened (token, head) pairs of a tile of
// tokens of one sequence; a workgroup takes 16*MT of them, all of which read
// the same cached rows.  Wave w forms the scores of 16 query rows x 16 keys
// (mt = w % MT, kb = w / MT); then every wave takes the softmax of all query
// rows for itself, in the layout of the value product's operand, and forms the
// output columns 16*(w + n*NW).
//   q_lat [rows, H, rank], q [rows, H, QP] with the rotated part at q_rot
//   tile_* null: decoding, tile i is row i of sequence i at ctx[i] - 1
//   NS > 1: partials part_m/part_l [rows, H, NS], part_acc [.., rank]
//   pages of 2^bs_log tokens
// Grid: (tiles, ceil(max tokens * H / (16*MT)), NS); block 64*NW.
// ---------------------------------------------------------------------------
template <int MT> constexpr int latent_waves() { return 2 * MT; }

template <int RP, int MT>
__global__ void __launch_bounds__(64 * latent_waves<MT>(), 2)
latent_tile_kernel(bf16 *__restrict__ out, float *__restrict__ part_m,
                   float *__restrict__ part_l, float *__restrict__ part_acc,
                   const bf16 *__restrict__ q_lat, const bf16 *__restrict__ q,
                   const bf16 *__restrict__ pool, const int *__restrict__ bt,
                   const int *__restrict__ ctx,
                   const int *__restrict__ tile_q0,
                   const int *__restrict__ tile_qn,
                   const int *__restrict__ tile_seq,
                   const int *__restrict__ tile_pos0,
                   const float *__restrict__ sink, float scale, int H,
                   int rank, int rot, int QP, int q_rot, int bs_log,
                   int MAXB, int NS) {
  constexpr int NW = latent_waves<MT>();
  constexpr int NT = 64 * NW;
  constexpr int KC = 16 * NW / MT;             // keys per step: at most 64
  constexpr int RT = 64;                       // room for the rotated part
  constexpr int SS = KC + 4;
  constexpr int NQ = RP / 32, NQR = RT / 32, KK = KC / 32;
  constexpr int NB = (RP / 16 + NW - 1) / NW;  // output blocks per wave
  // Keys in LDS: blocks of 64 columns, [KC keys][8 vectors] each; vector v of
  // key r lies at v ^ swizzle(r), so that neither the rows of a column nor the
  // columns of a row meet in a bank.  A copy moves 8 keys of a block.
  constexpr int CB = (RP + RT) / 64, BLOCK = KC * 64;
  constexpr int KG = KC / 8, IT = (CB + NW / KG - 1) / (NW / KG);
  __shared__ __align__(16) bf16 k_s[2][CB * BLOCK];
  __shared__ __align__(16) float s_s[MT * 16 * SS];

  const int tile = blockIdx.x;
  const int q0 = tile_q0 ? tile_q0[tile] : tile;
  const int qn = tile_q0 ? tile_qn[tile] : 1;
  const int seq = tile_q0 ? tile_seq[tile] : tile;
  const int pos0 = tile_q0 ? tile_pos0[tile] : ctx[tile] - 1;
  const int f0 = blockIdx.y * MT * 16;         // first flattened row
  if (f0 >= qn * H) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int l15 = lane & 15, g = lane >> 4;
  const int mt = wave % MT, kb = wave / MT;

  const int kv = pos0 + qn;
  const int per = ((kv + KC - 1) / KC + NS - 1) / NS * KC;
  const int t0 = min(kv, (int)blockIdx.z * per);
  const int t1 = min(kv, t0 + per);

  int last[4];                                 // last key of a score row
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int f = f0 + mt * 16 + g * 4 + r;
    last[r] = f < qn * H ? min(pos0 + f / H, t1 - 1) : -1;
  }
  float m[MT], l[MT];                          // of row a*16 + l15
#pragma unroll
  for (int a = 0; a < MT; ++a) {
    const int f = f0 + a * 16 + l15;
    const bool start = f < qn * H && sink && blockIdx.z == 0;
    m[a] = start ? sink[f % H] : -INFINITY;
    l[a] = start ? 1.f : 0.f;
  }
  // columns behind the latent and behind the rotated part stay zero, keys
  // behind the end finite
  if (rank < RP || rot < RT || t1 - t0 < 2 * KC) {
    for (int i = tid; i < CB * BLOCK / 4; i += NT)
      reinterpret_cast<uint4 *>(k_s)[i] = make_uint4(0, 0, 0, 0);
    __syncthreads();
  }

  // Q fragments: row l15 of this wave's 16, k = g*8 + i; rows that are not
  // there repeat the last one
  la_b16x8 qf[NQ + NQR];
  {
    const int f = min(f0 + mt * 16 + l15, qn * H - 1);
    const long row = (long)(q0 + f / H) * H + f % H;
    const bf16 *lp = q_lat + row * rank + g * 8;
    const bf16 *rp = q + row * QP + q_rot + g * 8;
#pragma unroll
    for (int kk = 0; kk < NQ; ++kk) {
      la_b16x8 v = {};
      if ((RP > 64 && kk < NQ / 2) || kk * 32 + g * 8 < rank)
        v = *reinterpret_cast<const la_b16x8 *>(lp + kk * 32);
      qf[kk] = v;
    }
#pragma unroll
    for (int kk = 0; kk < NQR; ++kk) {
      la_b16x8 v = {};
      if (kk * 32 + g * 8 < rot)
        v = *reinterpret_cast<const la_b16x8 *>(rp + kk * 32);
      qf[NQ + kk] = v;
    }
  }

  la_f32x4 o[MT][NB];
#pragma unroll
  for (int a = 0; a < MT; ++a)
#pragma unroll
    for (int n = 0; n < NB; ++n) o[a][n] = (la_f32x4){0.f, 0.f, 0.f, 0.f};

  // This lane copies vector `unit` of key `key` of a step.  Pool rows are
  // looked up a step ahead of the copies; -1 behind the end.
  const int width = rank + rot;
  const int key = wave % KG * 8 + (lane >> 3);
  const int unit = (lane & 7) ^ (key >> 1 & 7);
  const int *table = bt + (long)seq * MAXB;
  auto find = [&](int start) {
    const int token = start + key;
    return token < t1 ? (table[token >> bs_log] << bs_log) +
                            (token & ((1 << bs_log) - 1))
                      : -1;
  };
  auto fetch = [&](int at, bf16 *to) {
    if (at < 0) return;
    const bf16 *from = pool + (long)at * width + unit * 8;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int cb = wave / KG + it * (NW / KG), d = cb * 64 + unit * 8;
      if (CB % (NW / KG) && cb >= CB) continue;
      // more than half of the columns are always there (RP > 64)
      const bool sure = RP > 64 && (it + 1) * (NW / KG) * 64 <= RP / 2;
      if (sure || (d < RP ? d < rank : d - RP < rot))
        hyb::dma16(from + (cb * 64 < RP ? cb * 64 : rank),
                  to + cb * BLOCK + wave % KG * 512);
    }
  };
  // where this lane reads: the score operand (key kb*16 + l15, even and odd
  // 32-column steps) and the value operand (keys g*8 + l15/4 and 4 behind)
  const int sw = l15 >> 1;
  const int s_at[2] = {(kb * 16 + l15) * 64 + (g ^ sw) * 8,
                       (kb * 16 + l15) * 64 + ((4 + g) ^ sw) * 8};
  const int v_key = g * 8 + (l15 >> 2), v_unit = wave % 4 * 2 + (l15 >> 1 & 1);
  const int v_at[2] = {
      wave / 4 * BLOCK + v_key * 64 + (v_unit ^ (v_key >> 1 & 7)) * 8 +
          (l15 & 1) * 4,
      wave / 4 * BLOCK + (v_key + 4) * 64 +
          (v_unit ^ ((v_key + 4) >> 1 & 7)) * 8 + (l15 & 1) * 4};

  fetch(find(t0), k_s[0]);
  int at = find(t0 + KC);
  for (int start = t0, buf = 0; start < t1; start += KC, buf ^= 1) {
    hyb::dma_barrier();
    if (start + KC < t1) {
      fetch(at, k_s[buf ^ 1]);
      at = find(start + 2 * KC);
    }
    {
      la_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      const bf16 *kp = k_s[buf];
#pragma unroll
      for (int kk = 0; kk < NQ + NQR; ++kk)
        if (kk <= NQ || (kk - NQ) * 32 < rot)
          acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              qf[kk],
              *reinterpret_cast<const la_b16x8 *>(kp + kk / 2 * BLOCK +
                                                  s_at[kk & 1]),
              acc, 0, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        s_s[(mt * 16 + g * 4 + r) * SS + kb * 16 + l15] =
            start + kb * 16 + l15 <= last[r] ? acc[r] * scale : -INFINITY;
    }
    hyb::lds_barrier();
    la_b16x8 hi[MT][KK], lo[MT][KK];
#pragma unroll
    for (int a = 0; a < MT; ++a) {
      float p[KK][8], top = -INFINITY, sum = 0.f;
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) {
        hyb::load_v<8>(s_s + (a * 16 + l15) * SS + kk * 32 + g * 8, p[kk]);
#pragma unroll
        for (int j = 0; j < 8; ++j) top = fmaxf(top, p[kk][j]);
      }
      top = fmaxf(top, __shfl_xor(top, 16, 64));
      top = fmaxf(top, __shfl_xor(top, 32, 64));
      const float mn = fmaxf(m[a], top);
      const float alpha = m[a] == -INFINITY ? 0.f : __expf(m[a] - mn);
      const float base = mn == -INFINITY ? 0.f : mn;
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) {
        uint4 h4, l4;
        unsigned int *hp = &h4.x, *lp = &l4.x;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float u = __expf(p[kk][2 * j] - base);
          const float v = __expf(p[kk][2 * j + 1] - base);
          sum += u + v;
          hp[j] = pack_bf16x2(u, v);
          float uh, vh;
          unpack_bf16x2(hp[j], uh, vh);
          lp[j] = pack_bf16x2(u - uh, v - vh);
        }
        hi[a][kk] = __builtin_bit_cast(la_b16x8, h4);
        lo[a][kk] = __builtin_bit_cast(la_b16x8, l4);
      }
      sum += __shfl_xor(sum, 16, 64);
      sum += __shfl_xor(sum, 32, 64);
      l[a] = l[a] * alpha + sum;
      m[a] = mn;
      if (__any(alpha != 1.f)) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float w = __shfl(alpha, g * 4 + r, 64);
#pragma unroll
          for (int n = 0; n < NB; ++n) o[a][n][r] *= w;
        }
      }
    }
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) {
#pragma unroll
      for (int n = 0; n < NB; ++n) {
        const int col = (wave + n * NW) * 16;
        if (RP / 16 % NW && col >= RP) continue;
        // B fragment: column l15, keys g*8 + i
        const bf16 *vp = k_s[buf] + kk * 32 * 64 + n * (NW / 4) * BLOCK;
        const la_b16x8 v = la::join4(la::read_tr(vp + v_at[0]),
                                     la::read_tr(vp + v_at[1]));
#pragma unroll
        for (int a = 0; a < MT; ++a) {
          o[a][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi[a][kk], v,
                                                            o[a][n], 0, 0, 0);
          o[a][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo[a][kk], v,
                                                            o[a][n], 0, 0, 0);
        }
      }
    }
  }
#pragma unroll
  for (int a = 0; a < MT; ++a) {
    const float inv_a = l[a] > 0.f ? 1.f / l[a] : 0.f;
    const int fl = f0 + a * 16 + l15;
    if (NS > 1 && wave == 0 && g == 0 && fl < qn * H) {
      const long row = (long)(q0 + fl / H) * H + fl % H;
      part_m[row * NS + blockIdx.z] = m[a];
      part_l[row * NS + blockIdx.z] = l[a];
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float inv = __shfl(inv_a, g * 4 + r, 64);
      const int f = f0 + a * 16 + g * 4 + r;
      if (f >= qn * H) continue;
      const long row = (long)(q0 + f / H) * H + f % H;
#pragma unroll
      for (int n = 0; n < NB; ++n) {
        const int col = (wave + n * NW) * 16 + l15;
        if (col >= rank) continue;
        if (NS > 1)
          part_acc[(row * NS + blockIdx.z) * rank + col] = o[a][n][r];
        else
          out[row * rank + col] = f2bf(o[a][n][r] * inv);
      }
    }
  }
}

// Join the NS partial softmaxes of a row: a workgroup takes 128 columns, each
// of its four groups of 32 lanes every fourth part.
// Grid: (rows, H, ceil(rank / 128)); block 128; dynamic LDS NS floats.
__global__ void __launch_bounds__(128)
latent_combine_kernel(bf16 *__restrict__ out, const float *__restrict__ part_m,
                      const float *__restrict__ part_l,
                      const float *__restrict__ part_acc, int H, int rank,
                      int NS) {
  extern __shared__ float w_s[];
  __shared__ float scratch[2];
  __shared__ __align__(16) float sum_s[4][128];
  const long row = (long)blockIdx.x * H + blockIdx.y, base = row * NS;
  const float m = la::part_max(part_m, base, 1, NS, scratch);
  float l = 0.f;
  for (int i = threadIdx.x; i < NS; i += 128) {
    const float mi = part_m[base + i];
    const float w = mi == -INFINITY ? 0.f : __expf(mi - m);
    w_s[i] = w;
    l += w * part_l[base + i];
  }
  l = block_sum(l, scratch);                   // its barriers publish w_s
  const float inv = l > 0.f ? 1.f / l : 0.f;
  const int grp = threadIdx.x >> 5, c = (threadIdx.x & 31) * 4;
  const int d = blockIdx.z * 128 + c;
  float o[4] = {0.f, 0.f, 0.f, 0.f}, v[4];
  if (d < rank) {
#pragma unroll 4
    for (int i = grp; i < NS; i += 4) {
      hyb::load_v<4>(part_acc + (base + i) * rank + d, v);
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] = fmaf(w_s[i], v[j], o[j]);
    }
  }
  hyb::store_v<4>(&sum_s[grp][c], o);
  __syncthreads();
  if (grp || d >= rank) return;
#pragma unroll
  for (int j = 0; j < 4; ++j)
    o[j] = (o[j] + sum_s[1][c + j] + sum_s[2][c + j] + sum_s[3][c + j]) * inv;
  hyb::store_v<4>(out + row * rank + d, o);
}

// ---------------------------------------------------------------------------
// Latent space on the vector ALU: any size, bf16 or float32.  Row r belongs to
// sequence row_seq[r] and sits at row_pos[r].
// Grid: (rows, H); block 128; dynamic LDS 2 * rank + rot floats.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(128)
latent_rows_kernel(T *__restrict__ out, const T *__restrict__ q_lat,
                   const T *__restrict__ q, const T *__restrict__ pool,
                   const int *__restrict__ bt, const int *__restrict__ row_seq,
                   const int *__restrict__ row_pos,
                   const float *__restrict__ sink, float scale, int H,
                   int rank, int rot, int QP, int q_rot, int BS, int MAXB) {
  extern __shared__ float dyn_s[];
  float *q_s = dyn_s, *acc_s = dyn_s + rank + rot;
  __shared__ float p_s[128];
  __shared__ long at_s[128];
  __shared__ float scratch[2];
  const int h = blockIdx.y, tid = threadIdx.x, width = rank + rot;
  const long row = (long)blockIdx.x * H + h;
  const int pos = row_pos[blockIdx.x], seq = row_seq[blockIdx.x];
  for (int d = tid; d < width; d += 128)
    q_s[d] = hyb::to_f(d < rank ? q_lat[row * rank + d]
                                : q[row * QP + q_rot + d - rank]);
  for (int d = tid; d < rank; d += 128) acc_s[d] = 0.f;
  __syncthreads();
  float m = sink ? sink[h] : -INFINITY;
  float l = sink ? 1.f : 0.f;
  for (int start = 0; start <= pos; start += 128) {
    const int n = min(128, pos + 1 - start);
    float s = -INFINITY;
    if (tid < n) {
      const int token = start + tid;
      const long at =
          ((long)bt[(long)seq * MAXB + token / BS] * BS + token % BS) * width;
      at_s[tid] = at;
      float dot = 0.f;
      for (int d = 0; d < width; d += 4) {
        float v[4];
        hyb::load_v<4>(pool + at + d, v);
#pragma unroll
        for (int j = 0; j < 4; ++j) dot = fmaf(q_s[d + j], v[j], dot);
      }
      s = dot * scale;
    }
    const float mn = fmaxf(m, block_max(s, scratch));
    const float alpha = m == -INFINITY ? 0.f : expf(m - mn);
    const float p = tid < n ? expf(s - mn) : 0.f;
    p_s[tid] = p;
    l = l * alpha + block_sum(p, scratch);     // its barriers publish p_s
    m = mn;
    for (int d = tid; d < rank; d += 128) {
      float a = acc_s[d] * alpha;
      for (int t = 0; t < n; ++t)
        a = fmaf(p_s[t], hyb::to_f(pool[at_s[t] + d]), a);
      acc_s[d] = a;
    }
    __syncthreads();
  }
  for (int d = tid; d < rank; d += 128)
    hyb::put(out + row * rank + d, acc_s[d] / l);
}

// dst[r] = pool row of slots[r].  Grid: (rows); block 64.
__global__ void __launch_bounds__(64)
gather_latents_kernel(bf16 *__restrict__ dst, const bf16 *__restrict__ pool,
                      const int *__restrict__ slots, int width) {
  const uint4 *src = reinterpret_cast<const uint4 *>(
      pool + (long)slots[blockIdx.x] * width);
  uint4 *to = reinterpret_cast<uint4 *>(dst + (long)blockIdx.x * width);
  for (int i = threadIdx.x; i < width / 8; i += 64) to[i] = src[i];
}

// ---------------------------------------------------------------------------
// Expanded keys and values: 128 query rows of one head, 4 waves that own 32
// each.  Scores are formed transposed (keys x queries), so a lane holds one
// query: the softmax is in registers and its weights are the value product's
// operand as they lie (a matrix step's 16 keys are taken in the order the
// scores have; the values are read in the same order).
//   q [rows, H, QP]: dim plain, then rot rotated dimensions
//   ctx [n, rank + rot]: gathered latents, the rotated part at `rank`
//   kv [n, kv_w]: head h's keys at h*dim, its values at H*dim + h*vdim
//   NS > 1: partials part_m/part_l [tiles, H, NS, 128], part_acc [.., vdim]
// Grid: (tiles * H, NS); block 256.  DQ >= dim + rot, DV >= vdim.
// ---------------------------------------------------------------------------
template <int DQ, int DV>
__global__ void __launch_bounds__(256, DQ > 192 ? 1 : 2)
expanded_prefill_kernel(
    bf16 *__restrict__ out, float *__restrict__ part_m,
    float *__restrict__ part_l, float *__restrict__ part_acc,
    const bf16 *__restrict__ q, const bf16 *__restrict__ ctx,
    const bf16 *__restrict__ kv, const int *__restrict__ tile_q0,
    const int *__restrict__ tile_qn, const int *__restrict__ tile_pos0,
    const int *__restrict__ tile_ctx0, const float *__restrict__ sink,
    float scale, int tiles, int H, int dim, int rot, int vdim, int rank,
    int NS) {
  constexpr int KC = 64, KS = DQ + 8, VS = DV + 16;
  constexpr int NQ = DQ / 16, NB = DV / 32;
  constexpr int NK = KC * DQ / 8 / 256, NV = KC * DV / 8 / 256;
  __shared__ __align__(16) bf16 k_s[KC * KS];
  __shared__ __align__(16) bf16 v_s[KC * VS];
  // workgroups go round the 8 dies: keep a head's tiles on one, the long ones
  // (late rows) first
  int head, tile;
  {
    const int i = blockIdx.x;
    if (H % 8 == 0) {
      head = i % 8 + i / 8 / tiles * 8;
      tile = i / 8 % tiles;
    } else {
      head = i / tiles;
      tile = i % tiles;
    }
    tile = tiles - 1 - tile;
  }
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int l31 = lane & 31, half = lane >> 5, l15 = lane & 15;
  const int q0 = tile_q0[tile], qn = tile_qn[tile], pos0 = tile_pos0[tile];
  const int QP = dim + rot, width = rank + rot;
  const long kv_w = (long)H * (dim + vdim);
  const bf16 *cp = ctx + (long)tile_ctx0[tile] * width + rank;
  const bf16 *kp = kv + tile_ctx0[tile] * kv_w + (long)head * dim;
  const bf16 *vp = kv + tile_ctx0[tile] * kv_w + (long)H * dim +
                   (long)head * vdim;

  int begin = 0, limit = pos0 + qn;
  if (NS > 1) {
    const int per = ((limit + KC - 1) / KC + NS - 1) / NS * KC;
    begin = min(limit, (int)blockIdx.y * per);
    limit = min(limit, begin + per);
  }
  const int qr = wave * 32 + l31;              // this lane's query row
  const int last = pos0 + min(qr, qn - 1);     // last key it sees
  const int wave_last = pos0 + min(wave * 32 + 31, qn - 1);

  la_b16x8 qf[NQ];
#pragma unroll
  for (int kk = 0; kk < NQ; ++kk) {
    la_b16x8 v = {};
    const int d = kk * 16 + half * 8;
    if (qr < qn && d < QP)
      v = *reinterpret_cast<const la_b16x8 *>(
          q + ((long)(q0 + qr) * H + head) * QP + d);
    qf[kk] = v;
  }
  la_f32x16 o[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[b][r] = 0.f;
  const bool start_sink = sink && blockIdx.y == 0;
  float m = start_sink ? sink[head] : -INFINITY;
  float l = start_sink ? 1.f : 0.f;

  uint4 kr[NK], vr[NV];
  auto load = [&](int start) {
#pragma unroll
    for (int it = 0; it < NK; ++it) {
      const int i = tid + it * 256, key = i / (DQ / 8), d = i % (DQ / 8) * 8;
      const long t = start + key;
      uint4 v = make_uint4(0, 0, 0, 0);
      if (t < limit) {
        if (d < dim) v = *reinterpret_cast<const uint4 *>(kp + t * kv_w + d);
        else if (d < QP)
          v = *reinterpret_cast<const uint4 *>(cp + t * width + d - dim);
      }
      kr[it] = v;
    }
#pragma unroll
    for (int it = 0; it < NV; ++it) {
      const int i = tid + it * 256, key = i / (DV / 8), d = i % (DV / 8) * 8;
      const long t = start + key;
      vr[it] = t < limit && d < vdim
                   ? *reinterpret_cast<const uint4 *>(vp + t * kv_w + d)
                   : make_uint4(0, 0, 0, 0);
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int it = 0; it < NK; ++it) {
      const int i = tid + it * 256;
      *reinterpret_cast<uint4 *>(k_s + i / (DQ / 8) * KS +
                                 i % (DQ / 8) * 8) = kr[it];
    }
#pragma unroll
    for (int it = 0; it < NV; ++it) {
      const int i = tid + it * 256;
      *reinterpret_cast<uint4 *>(v_s + i / (DV / 8) * VS +
                                 i % (DV / 8) * 8) = vr[it];
    }
  };

  load(begin);
  for (int start = begin; start < limit; start += KC) {
    stage();
    __syncthreads();
    if (start + KC < limit) load(start + KC);
    if (start <= wave_last) {                  // wave-uniform
      la_f32x16 s[2];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
#pragma unroll
        for (int r = 0; r < 16; ++r) s[kb][r] = 0.f;
#pragma unroll
        for (int kk = 0; kk < NQ; ++kk)
          s[kb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
              *reinterpret_cast<const la_b16x8 *>(
                  k_s + (kb * 32 + l31) * KS + kk * 16 + half * 8),
              qf[kk], s[kb], 0, 0, 0);
      }
      // key of register r: kb*32 + (r & 3) + 8*(r >> 2) + 4*half
      float top = -INFINITY;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = start + kb * 32 + (r & 3) + 8 * (r >> 2) + 4 * half;
          const float v = key <= last && key < limit ? s[kb][r] * scale
                                                     : -INFINITY;
          s[kb][r] = v;
          top = fmaxf(top, v);
        }
      top = fmaxf(top, __shfl_xor(top, 32, 64));
      const float mn = fmaxf(m, top);
      const float alpha = m == -INFINITY ? 0.f : __expf(m - mn);
      const float base = mn == -INFINITY ? 0.f : mn;
      float sum = 0.f;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          s[kb][r] = __expf(s[kb][r] - base);
          sum += s[kb][r];
        }
      sum += __shfl_xor(sum, 32, 64);
      l = l * alpha + sum;
      m = mn;
      if (__any(alpha != 1.f)) {
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[b][r] *= alpha;
      }
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
#pragma unroll
        for (int st = 0; st < 2; ++st) {
          // slots 0-3 and 4-7 of a lane: keys 16*st + 4*half + 0..3 and + 8
          uint4 hi, lo;
          unsigned int *hp = &hi.x, *lp = &lo.x;
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float a = s[kb][8 * st + 2 * j];
            const float c = s[kb][8 * st + 2 * j + 1];
            hp[j] = pack_bf16x2(a, c);
            float ah, ch;
            unpack_bf16x2(hp[j], ah, ch);
            lp[j] = pack_bf16x2(a - ah, c - ch);
          }
          const la_b16x8 ph = __builtin_bit_cast(la_b16x8, hi);
          const la_b16x8 pl = __builtin_bit_cast(la_b16x8, lo);
          const bf16 *at = v_s +
                           (kb * 32 + st * 16 + half * 4 + (l15 >> 2)) * VS +
                           (lane >> 4 & 1) * 16 + (l15 & 3) * 4;
#pragma unroll
          for (int b = 0; b < NB; ++b) {
            const la_b16x8 v = la::join4(la::read_tr(at + b * 32),
                                         la::read_tr(at + 8 * VS + b * 32));
            o[b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v, ph, o[b], 0, 0,
                                                           0);
            o[b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v, pl, o[b], 0, 0,
                                                           0);
          }
        }
    }
    __syncthreads();
  }
  if (qr >= qn) return;
  // output column of register r: b*32 + (r & 3) + 8*(r >> 2) + 4*half
  if (NS > 1) {
    const long at = (((long)tile * H + head) * NS + blockIdx.y) * 128 + qr;
    if (half == 0) {
      part_m[at] = m;
      part_l[at] = l;
    }
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = b * 32 + 8 * j + 4 * half;
        if (d < vdim)
          *reinterpret_cast<float4 *>(part_acc + at * vdim + d) =
              make_float4(o[b][4 * j], o[b][4 * j + 1], o[b][4 * j + 2],
                          o[b][4 * j + 3]);
      }
    return;
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = b * 32 + 8 * j + 4 * half;
      if (d >= vdim) continue;
      float v[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = o[b][4 * j + e] * inv;
      hyb::store_v<4>(out + ((long)(q0 + qr) * H + head) * vdim + d, v);
    }
}

// Grid: (tiles, H, 128); block 64.
__global__ void __launch_bounds__(64)
expanded_combine_kernel(bf16 *__restrict__ out,
                        const float *__restrict__ part_m,
                        const float *__restrict__ part_l,
                        const float *__restrict__ part_acc,
                        const int *__restrict__ tile_q0,
                        const int *__restrict__ tile_qn, int H, int vdim,
                        int NS) {
  const int tile = blockIdx.x, h = blockIdx.y, qi = blockIdx.z;
  if (qi >= tile_qn[tile]) return;
  const long base = ((long)tile * H + h) * NS * 128 + qi;
  float m = -INFINITY;
  for (int i = 0; i < NS; ++i) m = fmaxf(m, part_m[base + i * 128]);
  const int d = threadIdx.x * 4;
  float l = 0.f, o[4] = {0.f, 0.f, 0.f, 0.f}, v[4];
  for (int i = 0; i < NS; ++i) {
    const long at = base + i * 128;
    const float mi = part_m[at];
    if (mi == -INFINITY) continue;
    const float w = __expf(mi - m);
    l = fmaf(w, part_l[at], l);
    if (d < vdim) {
      hyb::load_v<4>(part_acc + at * vdim + d, v);
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] = fmaf(w, v[j], o[j]);
    }
  }
  if (d >= vdim) return;
  const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] *= inv;
  hyb::store_v<4>(out + ((long)(tile_q0[tile] + qi) * H + h) * vdim + d, o);
}
