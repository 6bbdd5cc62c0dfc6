// The two paged-attention bodies that more than one model family launches:
// the 128-row T12 prefill tile and the matrix-core flash-decode.
//
//   DP     head dimension the tile is built for (64 or 128)
//   LOCAL  false: causal softmax attention, head dimension exactly DP.
//          true:  head dimension D <= DP (multiple of 8, zero-padded in the
//                 tile), optionally confined to position chunks, optionally
//                 with one added to the softmax denominator, and with the
//                 probabilities fed to the matrix cores as a bf16 pair
//                 (hi + lo), so that they keep 16 significant bits.
//   chunk  LOCAL: query i sees key j <= i only if i / chunk == j / chunk,
//          both counted from the start of the sequence; 0 = unconfined.
//   sink   LOCAL: the running softmax of a row starts from a key of score 0
//          that has no value (m = 0, l = 1) instead of from nothing.
//
// Fragment maps (16x16x32 bf16 MFMA):
//   A: row = lane&15,           k = (lane>>4)*8 + i   (8 contiguous)
//   B: col = lane&15,           k = (lane>>4)*8 + i
//   C/D: col = lane&15,         row = (lane>>4)*4 + reg
#pragma once

#include "common.h"

#define MF_KCHUNK 64
#define MF_QT 16
#define MF_D 128

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4_t __attribute__((ext_vector_type(4)));
typedef float f32x4_t __attribute__((ext_vector_type(4)));

namespace attn_core {

// Element offset of column d in an XOR-swizzled [row][DP] LDS image: the 16
// rows of a fragment read land in different 16-byte bank groups.
template <int DP>
__device__ __forceinline__ int swz(int row, int d) {
  if constexpr (DP >= 128) return d ^ ((row & 15) << 3);
  return d ^ (((row >> 1) & 7) << 3);
}

// Two C-layout key blocks of a transposed score tile (lane: query row =
// lane&15, keys (lane>>4)*4 + reg of each block) -> the A fragment of those
// 32 keys (lane: row = lane&15, keys (lane>>4)*8 + i): pack to bf16 dwords,
// then a permlane32 + permlane16 swap pair.
__device__ __forceinline__ bf16x8_t scores_to_afrag(const f32x4_t &s0,
                                                    const f32x4_t &s1) {
  unsigned int d0 = pack_bf16x2(s0[0], s0[1]);
  unsigned int d1 = pack_bf16x2(s0[2], s0[3]);
  unsigned int e0 = pack_bf16x2(s1[0], s1[1]);
  unsigned int e1 = pack_bf16x2(s1[2], s1[3]);
  {
    auto r = __builtin_amdgcn_permlane32_swap(d0, e0, false, false);
    d0 = r[0]; e0 = r[1];
  }
  {
    auto r = __builtin_amdgcn_permlane32_swap(d1, e1, false, false);
    d1 = r[0]; e1 = r[1];
  }
  {
    auto r = __builtin_amdgcn_permlane16_swap(d0, e0, false, false);
    d0 = r[0]; e0 = r[1];
  }
  {
    auto r = __builtin_amdgcn_permlane16_swap(d1, e1, false, false);
    d1 = r[0]; e1 = r[1];
  }
  const uint4 av = make_uint4(d0, d1, e0, e1);
  return __builtin_bit_cast(bf16x8_t, av);
}

// What bf16 rounding leaves of a score block.
__device__ __forceinline__ f32x4_t bf16_rest(const f32x4_t &s) {
  f32x4_t r;
#pragma unroll
  for (int i = 0; i < 4; ++i) r[i] = s[i] - bf2f(f2bf(s[i]));
  return r;
}

// ---------------------------------------------------------------------------
// T12 prefill tile: 128 query rows, 8 waves, each wave OWNS one 16-row
// qblock end to end.  Swapped QK^T (mfma(K, Q)) makes every S row lane-local,
// so the online softmax runs fully in registers; two barriers per 64-key
// chunk (staging).
//   K: XOR-swizzled [64][DP] image;  V: row-major [64][DP + 6] image.
// Grid: (tiles of 128 rows, Hq, NS); block 512.  NS > 1 (LOCAL only)
// partitions the key walk and writes unnormalised partials
//   part_m/part_l: [tiles, Hq, NS, 128] f32, part_acc: [..., D] f32.
// ---------------------------------------------------------------------------
template <int DP, bool LOCAL>
__device__ __forceinline__ void prefill_t12(
    bf16 *__restrict__ out, float *__restrict__ part_m,
    float *__restrict__ part_l, float *__restrict__ part_acc,
    const bf16 *__restrict__ q, const bf16 *__restrict__ kc,
    const bf16 *__restrict__ vc, const int *__restrict__ bt,
    const int *__restrict__ tile_q0, const int *__restrict__ tile_qn,
    const int *__restrict__ tile_seq, const int *__restrict__ tile_pos0,
    float scale, int Hq, int Hkv, int BS, int MAXB, int GQ, int NS, int Drt,
    int chunk, bool sink) {
  constexpr int VRS = DP + 6;        // odd dword stride: bank spread
  constexpr int NK = DP / 32;        // k-steps of QK^T
  constexpr int NB = DP / 16;        // output column blocks
  constexpr int IT = MF_KCHUNK * DP / 8 / 512;
  const int D = LOCAL ? Drt : DP;
  const int tile = blockIdx.x;
  const int h = blockIdx.y;
  const int hk = h / GQ;
  const int tid = threadIdx.x;
  const int wave = tid >> 6;
  const int lane = tid & 63;
  const int q0 = tile_q0[tile];
  const int qn = tile_qn[tile];
  const int seq = tile_seq[tile];
  const int pos0 = tile_pos0[tile];
  int kv_begin = 0, kv_limit = pos0 + qn;
  bool first_part = true;
  if constexpr (LOCAL) {
    if (chunk > 0) kv_begin = pos0 / chunk * chunk;
    if (NS > 1) {
      const int n64 = (kv_limit - kv_begin + MF_KCHUNK - 1) / MF_KCHUNK;
      const int per = (n64 + NS - 1) / NS * MF_KCHUNK;
      kv_begin += (int)blockIdx.z * per;
      kv_limit = min(kv_limit, kv_begin + per);
      first_part = blockIdx.z == 0;
    }
  }

  __shared__ bf16 k_s[MF_KCHUNK * DP];       // XOR-swizzled
  __shared__ bf16 v_s[MF_KCHUNK * VRS];      // row-major
  __shared__ float alpha_w[8][16];
  __shared__ float l_w[8][16];

  const int qr = lane & 15;                  // this lane's qrow (in qblock)
  const int g = lane >> 4;                   // 16-lane group
  const int row_local = wave * 16 + qr;      // row within the 128-row tile

  // Q B-fragments in registers: lane holds Q[qrow][k = g*8 + t] per kk
  bf16x8_t q_frag[NK];
#pragma unroll
  for (int kk = 0; kk < NK; ++kk) {
    bf16x8_t v = {};
    if (row_local < qn && (!LOCAL || kk * 32 + g * 8 < D))
      v = *reinterpret_cast<const bf16x8_t *>(
          q + ((long)(q0 + row_local) * Hq + h) * D + kk * 32 + g * 8);
    q_frag[kk] = v;
  }

  // per-lane online-softmax state for qrow (replicated over the 4
  // same-qrow lanes, deterministically identical)
  float m_run = -INFINITY, l_run = 0.f;
  if constexpr (LOCAL) {
    if (sink && first_part) { m_run = 0.f; l_run = 1.f; }
  }
  // O accumulators: C rows = qrows (g*4+r), col = d
  f32x4_t o_acc[NB];
#pragma unroll
  for (int db = 0; db < NB; ++db) o_acc[db] = (f32x4_t){0.f, 0.f, 0.f, 0.f};

  const long panel_stride = (long)Hkv * BS * D;
  const int abs_qrow = min(row_local, qn - 1) + pos0;   // causal bound
  const int low = (LOCAL && chunk > 0) ? abs_qrow / chunk * chunk : 0;

  uint4 kreg[IT], vreg[IT];
  auto issue_loads = [&](int start_, int limit_) {
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int i = tid + it * 512;
      const int key = (i * 8) / DP, d = (i * 8) % DP;
      uint4 kv = make_uint4(0, 0, 0, 0), vv = make_uint4(0, 0, 0, 0);
      const int token = start_ + key;
      if (token < limit_ && (!LOCAL || d < D)) {
        const long blk = bt[(long)seq * MAXB + token / BS];
        const long off =
            blk * panel_stride + ((long)hk * BS + token % BS) * D + d;
        kv = reinterpret_cast<const uint4 *>(kc + off)[0];
        vv = reinterpret_cast<const uint4 *>(vc + off)[0];
      }
      kreg[it] = kv;
      vreg[it] = vv;
    }
  };
  auto write_staged = [&]() {
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int i = tid + it * 512;
      const int key = (i * 8) / DP, d = (i * 8) % DP;
      reinterpret_cast<uint4 *>(k_s + key * DP + swz<DP>(key, d))[0] =
          kreg[it];
      const uint *vw = reinterpret_cast<const uint *>(&vreg[it]);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        reinterpret_cast<uint *>(v_s + key * VRS + d)[j] = vw[j];
    }
  };

  issue_loads(kv_begin, kv_limit);
  for (int start = kv_begin; start < kv_limit; start += MF_KCHUNK) {
    const int clen = min(MF_KCHUNK, kv_limit - start);
    write_staged();
    __syncthreads();
    if (start + MF_KCHUNK < kv_limit)
      issue_loads(start + MF_KCHUNK, kv_limit);

    // ---- S^T = K·Q^T per 16-key block: C[key][qrow], lane-local rows --
    f32x4_t s_frag[4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NK; ++kk) {
        // A = K rows (keys kb*16 + qr), k-slice g*8 (+kk*32), swizzled
        bf16x8_t a = *reinterpret_cast<const bf16x8_t *>(
            k_s + (kb * 16 + qr) * DP + swz<DP>(qr, kk * 32 + g * 8));
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, q_frag[kk], acc,
                                                      0, 0, 0);
      }
      s_frag[kb] = acc;
    }

    // ---- in-register online softmax over the 64-key chunk -----------
    // (masked scores, then P, overwrite s_frag in place — the S pipeline
    // must not triple register pressure: vals/pv/s_frag were 48 VGPRs)
    float mymax = -INFINITY;
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = kb * 16 + g * 4 + r;
        const int token = start + key;
        const bool ok = (token <= abs_qrow) && (key < clen) &&
                        (!LOCAL || token >= low);
        const float sv = ok ? s_frag[kb][r] * scale : -INFINITY;
        s_frag[kb][r] = sv;
        mymax = fmaxf(mymax, sv);
      }
    }
    mymax = fmaxf(mymax, __shfl_xor(mymax, 16));
    mymax = fmaxf(mymax, __shfl_xor(mymax, 32));
    // (T13 defer-max measured perf-neutral here at 3x the rounding error
    // — the rescale pass is only 32 VALU ops — so the exact path stays)
    const float mn = fmaxf(m_run, mymax);
    const float alpha = (m_run == -INFINITY) ? 0.f : __expf(m_run - mn);
    float psum = 0.f;
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p = (s_frag[kb][r] == -INFINITY || mn == -INFINITY)
                            ? 0.f : __expf(s_frag[kb][r] - mn);
        psum += p;
        s_frag[kb][r] = p;
      }
    }
    psum += __shfl_xor(psum, 16);
    psum += __shfl_xor(psum, 32);
    l_run = l_run * alpha + psum;
    m_run = mn;
    if (lane < 16) alpha_w[wave][lane] = alpha;   // qrow == lane here

    // ---- O rescale (alpha for PV C rows g*4+r via the wave strip) ----
#pragma unroll
    for (int db = 0; db < NB; ++db) {
#pragma unroll
      for (int r = 0; r < 4; ++r) o_acc[db][r] *= alpha_w[wave][g * 4 + r];
    }

    // ---- P -> A fragments + PV ---------------------------------------
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      const bf16x8_t a_frag =
          scores_to_afrag(s_frag[2 * kk], s_frag[2 * kk + 1]);
      bf16x8_t a_rest = {};
      if constexpr (LOCAL)
        a_rest = scores_to_afrag(bf16_rest(s_frag[2 * kk]),
                                 bf16_rest(s_frag[2 * kk + 1]));
#pragma unroll
      for (int db = 0; db < NB; ++db) {
        bf16x8_t b;
#pragma unroll
        for (int t = 0; t < 8; ++t)
          b[t] = v_s[(kk * 32 + g * 8 + t) * VRS + db * 16 + qr];
        o_acc[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_frag, b,
                                                            o_acc[db], 0, 0, 0);
        if constexpr (LOCAL)
          o_acc[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              a_rest, b, o_acc[db], 0, 0, 0);
      }
    }
    __syncthreads();   // next chunk restages k_s / v_s
  }

  if constexpr (LOCAL) {
    if (NS > 1) {
      const long base = (((long)tile * Hq + h) * NS + blockIdx.z) * 128;
      if (lane < 16) {
        part_m[base + wave * 16 + lane] = m_run;
        part_l[base + wave * 16 + lane] = l_run;
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = wave * 16 + g * 4 + r;
        if (row >= qn) continue;
#pragma unroll
        for (int db = 0; db < NB; ++db)
          if (db * 16 + qr < D)
            part_acc[(base + row) * D + db * 16 + qr] = o_acc[db][r];
      }
      return;
    }
  }

  if (lane < 16) l_w[wave][lane] = l_run;
  // epilogue: PV C rows = qrows g*4+r of this wave's qblock
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = wave * 16 + g * 4 + r;
    if (row >= qn) continue;
    const float lv = l_w[wave][g * 4 + r];
    const float denom = lv > 0.f ? lv : 1.f;
#pragma unroll
    for (int db = 0; db < NB; ++db)
      if (!LOCAL || db * 16 + qr < D)
        out[((long)(q0 + row) * Hq + h) * D + db * 16 + qr] =
            f2bf(o_acc[db][r] / denom);
  }
}

// ---------------------------------------------------------------------------
// Matrix-core flash-decode: the GQ query heads sharing one KV head are the
// first GQ rows of a 16-row Q tile (rest zero), K/V stream through LDS, both
// products run on the matrix cores, the context is split over NS workgroups.
//   part_m/part_l: [B, Hq, NS] f32;  part_acc: [B, Hq, NS, D] f32
// Grid: (B, Hkv, NS); block 256.  GQ <= 16.
// ---------------------------------------------------------------------------
template <int DP, bool LOCAL>
__device__ __forceinline__ void decode_mfma(
    float *__restrict__ part_m, float *__restrict__ part_l,
    float *__restrict__ part_acc, const bf16 *__restrict__ q,
    const bf16 *__restrict__ kc, const bf16 *__restrict__ vc,
    const int *__restrict__ bt, const int *__restrict__ ctx, float scale,
    int Hq, int Hkv, int BS, int MAXB, int GQ, int NS, int Drt, int chunk,
    bool sink) {
  constexpr int VRS = DP + 6;
  constexpr int SPS = MF_KCHUNK + 4;
  constexpr int VPS = MF_KCHUNK + 8;
  constexpr int NK = DP / 32;
  constexpr int NB = DP / 64;          // 16-column blocks per wave
  constexpr int IT = MF_KCHUNK * DP / 8 / 256;
  const int D = LOCAL ? Drt : DP;
  const int b = blockIdx.x;
  const int hk = blockIdx.y;
  const int split = blockIdx.z;
  const int tid = threadIdx.x;
  const int wave = tid >> 6;
  const int lane = tid & 63;
  const int len = ctx[b];
  // the token attends from position len - 1
  const int low = (LOCAL && chunk > 0) ? (len - 1) / chunk * chunk : 0;
  const int chunks = (len - low + MF_KCHUNK - 1) / MF_KCHUNK;
  const int per = (chunks + NS - 1) / NS;
  const int t0 = low + split * per * MF_KCHUNK;
  const int t1 = min(len, low + (split + 1) * per * MF_KCHUNK);
  const bool dead = (t0 >= len);
  const bool has_sink = LOCAL && sink && split == 0;

  // q_s/k_s: XOR-swizzled [row][DP] images
  __shared__ bf16 q_s[MF_QT * DP];
  __shared__ bf16 k_s[MF_KCHUNK * DP];
  __shared__ bf16 v_s[MF_KCHUNK * VRS];   // row-major V
  __shared__ float s_s[MF_QT * SPS];
  __shared__ bf16 p_s[MF_QT * VPS];
  __shared__ bf16 p_lo[LOCAL ? MF_QT * VPS : 1];
  __shared__ float m_s[MF_QT], l_s[MF_QT], alpha_s[MF_QT];

  // Q tile: rows 0..GQ-1 are this KV head's query heads, rest zero
  for (int i = tid; i < MF_QT * DP / 8; i += 256) {
    const int r = (i * 8) / DP, c = (i * 8) % DP;
    uint4 val = make_uint4(0, 0, 0, 0);
    if (r < GQ && (!LOCAL || c < D))
      val = reinterpret_cast<const uint4 *>(
          q + ((long)b * Hq + hk * GQ + r) * D + c)[0];
    reinterpret_cast<uint4 *>(q_s + r * DP + swz<DP>(r, c))[0] = val;
  }
  if (tid < MF_QT) {
    m_s[tid] = has_sink ? 0.f : -INFINITY;
    l_s[tid] = has_sink ? 1.f : 0.f;
  }
  __syncthreads();

  f32x4_t o_acc[NB];
#pragma unroll
  for (int n = 0; n < NB; ++n) o_acc[n] = (f32x4_t){0.f, 0.f, 0.f, 0.f};

  const long panel_stride = (long)Hkv * BS * D;
  const int a_row = lane & 15;
  const int a_koff = (lane >> 4) * 8;
  const int c_col = lane & 15;
  const int c_row0 = (lane >> 4) * 4;

  uint4 kreg[IT], vreg[IT];
  auto issue_loads = [&](int start_, int limit_) {
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int i = tid + it * 256;
      const int key = (i * 8) / DP, d = (i * 8) % DP;
      uint4 kv = make_uint4(0, 0, 0, 0), vv = make_uint4(0, 0, 0, 0);
      const int token = start_ + key;
      if (token < limit_ && (!LOCAL || d < D)) {
        const long blk = bt[(long)b * MAXB + token / BS];
        const long off =
            blk * panel_stride + ((long)hk * BS + token % BS) * D + d;
        kv = reinterpret_cast<const uint4 *>(kc + off)[0];
        vv = reinterpret_cast<const uint4 *>(vc + off)[0];
      }
      kreg[it] = kv;
      vreg[it] = vv;
    }
  };
  auto write_staged = [&]() {
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int i = tid + it * 256;
      const int key = (i * 8) / DP, d = (i * 8) % DP;
      reinterpret_cast<uint4 *>(k_s + key * DP + swz<DP>(key, d))[0] =
          kreg[it];
      const uint *vw = reinterpret_cast<const uint *>(&vreg[it]);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        reinterpret_cast<uint *>(v_s + key * VRS + d)[j] = vw[j];
    }
  };

  issue_loads(t0, t1);
  for (int start = t0; start < t1; start += MF_KCHUNK) {
    const int clen = min(MF_KCHUNK, t1 - start);
    write_staged();
    __syncthreads();
    if (start + MF_KCHUNK < t1)
      issue_loads(start + MF_KCHUNK, t1);

    // S = Q·K^T (wave w: key block w*16..w*16+15); no causal mask in decode
    {
      f32x4_t s_acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NK; ++kk) {
        bf16x8_t a = *reinterpret_cast<const bf16x8_t *>(
            q_s + a_row * DP + swz<DP>(a_row, kk * 32 + a_koff));
        bf16x8_t b2 = *reinterpret_cast<const bf16x8_t *>(
            k_s + (wave * 16 + a_row) * DP
                + swz<DP>(a_row, kk * 32 + a_koff));
        s_acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b2, s_acc, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = c_row0 + r;
        const int col = wave * 16 + c_col;
        s_s[row * SPS + col] = (col < clen) ? s_acc[r] * scale : -INFINITY;
      }
    }
    __syncthreads();

    // online softmax (16 threads per row)
    {
      const int row = tid >> 4;
      const int sub = tid & 15;
      float v0 = s_s[row * SPS + sub];
      float v1 = s_s[row * SPS + sub + 16];
      float v2 = s_s[row * SPS + sub + 32];
      float v3 = s_s[row * SPS + sub + 48];
      float mymax = fmaxf(fmaxf(v0, v1), fmaxf(v2, v3));
#pragma unroll
      for (int w = 8; w >= 1; w >>= 1)
        mymax = fmaxf(mymax, __shfl_xor(mymax, w, 16));
      const float m_old = m_s[row];
      const float mn = fmaxf(m_old, mymax);
      const float alpha = (m_old == -INFINITY) ? 0.f : __expf(m_old - mn);
      float p0 = (v0 == -INFINITY || mn == -INFINITY) ? 0.f : __expf(v0 - mn);
      float p1 = (v1 == -INFINITY || mn == -INFINITY) ? 0.f : __expf(v1 - mn);
      float p2 = (v2 == -INFINITY || mn == -INFINITY) ? 0.f : __expf(v2 - mn);
      float p3 = (v3 == -INFINITY || mn == -INFINITY) ? 0.f : __expf(v3 - mn);
      float psum = p0 + p1 + p2 + p3;
#pragma unroll
      for (int w = 8; w >= 1; w >>= 1)
        psum += __shfl_xor(psum, w, 16);
      if (sub == 0) {
        l_s[row] = l_s[row] * alpha + psum;
        m_s[row] = mn;
        alpha_s[row] = alpha;
      }
      p_s[row * VPS + sub] = f2bf(p0);
      p_s[row * VPS + sub + 16] = f2bf(p1);
      p_s[row * VPS + sub + 32] = f2bf(p2);
      p_s[row * VPS + sub + 48] = f2bf(p3);
      if constexpr (LOCAL) {
        p_lo[row * VPS + sub] = f2bf(p0 - bf2f(f2bf(p0)));
        p_lo[row * VPS + sub + 16] = f2bf(p1 - bf2f(f2bf(p1)));
        p_lo[row * VPS + sub + 32] = f2bf(p2 - bf2f(f2bf(p2)));
        p_lo[row * VPS + sub + 48] = f2bf(p3 - bf2f(f2bf(p3)));
      }
    }
    __syncthreads();

    // O rescale + O += P·V (wave w: output cols w*DP/4 .. + DP/4)
    {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float a = alpha_s[c_row0 + r];
#pragma unroll
        for (int n = 0; n < NB; ++n) o_acc[n][r] *= a;
      }
#pragma unroll
      for (int kk = 0; kk < MF_KCHUNK / 32; ++kk) {
        bf16x8_t a = *reinterpret_cast<const bf16x8_t *>(
            p_s + a_row * VPS + kk * 32 + a_koff);
        bf16x8_t a_rest = {};
        if constexpr (LOCAL)
          a_rest = *reinterpret_cast<const bf16x8_t *>(
              p_lo + a_row * VPS + kk * 32 + a_koff);
#pragma unroll
        for (int n = 0; n < NB; ++n) {
          bf16x8_t bv;
#pragma unroll
          for (int t = 0; t < 8; ++t)
            bv[t] = v_s[(kk * 32 + a_koff + t) * VRS + wave * (DP / 4)
                        + n * 16 + c_col];
          o_acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, bv, o_acc[n],
                                                             0, 0, 0);
          if constexpr (LOCAL)
            o_acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                a_rest, bv, o_acc[n], 0, 0, 0);
        }
      }
    }
    __syncthreads();
  }

  // partials out (unnormalized; a combine kernel joins the splits)
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = c_row0 + r;
    if (row >= GQ) continue;
    const int h = hk * GQ + row;
    const long base = ((long)b * Hq + h) * NS + split;
    if (c_col == 0 && wave == 0) {
      part_m[base] = (dead && !has_sink) ? -INFINITY : m_s[row];
      part_l[base] = (dead && !has_sink) ? 0.f : l_s[row];
    }
#pragma unroll
    for (int n = 0; n < NB; ++n) {
      const int col = wave * (DP / 4) + n * 16 + c_col;
      if (!LOCAL || col < D)
        part_acc[base * D + col] = dead ? 0.f : o_acc[n][r];
    }
  }
}

// ---------------------------------------------------------------------------
// Join NS split partials of one (row, head): the rows' partials lie `step`
// entries apart starting at `base0`.  Block of 128 threads, D <= 128.
// ---------------------------------------------------------------------------
__device__ __forceinline__ void combine_splits(
    bf16 *__restrict__ dst, const float *__restrict__ part_m,
    const float *__restrict__ part_l, const float *__restrict__ part_acc,
    long base0, long step, int D, int NS) {
  const int tid = threadIdx.x;
  __shared__ float scratch[8];
  float M = -INFINITY;
  for (int i = tid; i < NS; i += blockDim.x)
    M = fmaxf(M, part_m[base0 + i * step]);
  M = block_max(M, scratch);
  float L = 0.f;
  for (int i = tid; i < NS; i += blockDim.x) {
    const float mi = part_m[base0 + i * step];
    L += (mi == -INFINITY) ? 0.f : part_l[base0 + i * step] * __expf(mi - M);
  }
  L = block_sum(L, scratch);
  if (tid < D) {
    float o = 0.f;
    for (int i = 0; i < NS; ++i) {
      const float mi = part_m[base0 + i * step];
      if (mi == -INFINITY) continue;
      o = fmaf(part_acc[(base0 + i * step) * D + tid], __expf(mi - M), o);
    }
    dst[tid] = f2bf(L > 0.f ? o / L : 0.f);
  }
}

}  // namespace attn_core
