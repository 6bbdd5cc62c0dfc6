// Linear attention with a decaying matrix state (gfx950).
//
//   S_t = diag(a_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t * qscale
//
// per head, with S float32 of [dim, vdim].  Two kinds of decay:
//   CH = false  a_t is one constant per head;
//   CH = true   a_t is per token and key channel, given by its logarithm.
//
// The state pool is stored value-major, state[slot][head][v][d]: a lane then
// holds consecutive key channels of one value row, which is how the decode
// kernel reduces over d and how the matrix cores want the state as a B
// operand.  A sequence whose first row sits at position 0 starts from zero
// whatever its slot holds, so slots are reused without clearing.
//
// q, k and v are read in place from the rows of the fused input projection;
// `act` is applied to all three as they are loaded.
//
// Two paths:
//   * linear_recurrent: token by token, state rows in registers.  Decode (one
//     token per sequence), float32, and head sizes the tiles do not take.
//   * chunked (bf16 prefill, dim and vdim multiples of 8, dim <= 256):
//     sequences are cut into chunks of LIN_CHUNK tokens from where the batch
//     brings them in; linear_chunk_state forms every chunk's own contribution
//     to the state, linear_chunk_scan turns those into the state at each
//     chunk's start (and the final state into the pool), linear_chunk_out
//     forms the outputs.  q, k, v enter the matrix cores as bf16; everything
//     that holds a decay, a score or the state (float32) enters as a bf16
//     pair hi + lo with products hi*hi + hi*lo (+ lo*hi), accumulated in
//     float32.

#include "attention_core.h"
#include "hybrid_common.h"

#define LIN_CHUNK 64
#define LIN_TS (LIN_CHUNK + 8)    // LDS row stride of a [column][token] image

// ---------------------------------------------------------------------------
// Token-by-token form.  LPR lanes share one value row, each holding EPL
// groups of VEC channels; a workgroup covers 4 * 256/LPR value rows.
//   decay: CH ? log decay [rows, H*D] : decay [H]
//   seg_row0 null: sequence s is row s, one token.
// Grid: (sequences, H, ceil(V / (1024/LPR))); block 256.
// ---------------------------------------------------------------------------
template <typename T, int VEC, int LPR, int EPL, bool CH>
__global__ void __launch_bounds__(256)
linear_recurrent_kernel(T *__restrict__ o, const T *__restrict__ proj,
                        long stride, int q_off, int k_off, int v_off, int H,
                        int D, int V, int act, float qscale,
                        const float *__restrict__ decay,
                        float *__restrict__ state,
                        const int *__restrict__ seg_row0,
                        const int *__restrict__ seg_len,
                        const int *__restrict__ seg_slot,
                        const int *__restrict__ positions) {
  constexpr int RPG = 256 / LPR;     // value rows side by side
  constexpr int RPT = 4;             // value rows per thread
  constexpr int E = VEC * EPL;
  const int seg = blockIdx.x;
  const int h = blockIdx.y;
  const int tid = threadIdx.x;
  const int lane = tid % LPR;
  const int rg = tid / LPR;
  const int v_base = blockIdx.z * (RPG * RPT) + rg;
  const long row0 = seg_row0 ? seg_row0[seg] : seg;
  const int len = seg_row0 ? seg_len[seg] : 1;
  if (len <= 0) return;
  float *st = state + ((long)seg_slot[seg] * H + h) * (long)V * D;
  const bool fresh = positions[row0] == 0;

  float S[RPT][E];
#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int v = v_base + r * RPG;
#pragma unroll
    for (int e = 0; e < EPL; ++e) {
      const int d = (e * LPR + lane) * VEC;
#pragma unroll
      for (int i = 0; i < VEC; ++i) S[r][e * VEC + i] = 0.f;
      if (!fresh && v < V && d < D)
        hyb::load_v<VEC>(st + (long)v * D + d, S[r] + e * VEC);
    }
  }
  const float a_head = CH ? 0.f : decay[h];

  for (int t = 0; t < len; ++t) {
    const T *p = proj + (row0 + t) * stride;
    float q[E], k[E], a[E], v[RPT];
#pragma unroll
    for (int e = 0; e < EPL; ++e) {
      const int d = (e * LPR + lane) * VEC;
#pragma unroll
      for (int i = 0; i < VEC; ++i) {
        q[e * VEC + i] = 0.f;
        k[e * VEC + i] = 0.f;
        a[e * VEC + i] = a_head;
      }
      if (d < D) {
        hyb::load_v<VEC>(p + q_off + h * D + d, q + e * VEC);
        hyb::load_v<VEC>(p + k_off + h * D + d, k + e * VEC);
        if constexpr (CH) {
          hyb::load_v<VEC>(decay + ((row0 + t) * H + h) * (long)D + d,
                           a + e * VEC);
#pragma unroll
          for (int i = 0; i < VEC; ++i)
            a[e * VEC + i] = expf(a[e * VEC + i]);
        }
#pragma unroll
        for (int i = 0; i < VEC; ++i) {
          q[e * VEC + i] = hyb::activate<T>(q[e * VEC + i], act);
          k[e * VEC + i] = hyb::activate<T>(k[e * VEC + i], act);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      const int vi = v_base + r * RPG;
      v[r] = vi < V ? hyb::activate<T>(hyb::to_f(p[v_off + h * V + vi]), act)
                    : 0.f;
    }
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      float acc = 0.f;
#pragma unroll
      for (int i = 0; i < E; ++i) {
        S[r][i] = a[i] * S[r][i] + k[i] * v[r];
        acc = fmaf(q[i], S[r][i], acc);
      }
#pragma unroll
      for (int w = LPR / 2; w >= 1; w >>= 1) acc += __shfl_xor(acc, w, LPR);
      const int vi = v_base + r * RPG;
      if (lane == 0 && vi < V)
        hyb::put(o + ((row0 + t) * H + h) * (long)V + vi, acc * qscale);
    }
  }

#pragma unroll
  for (int r = 0; r < RPT; ++r) {
    const int v = v_base + r * RPG;
#pragma unroll
    for (int e = 0; e < EPL; ++e) {
      const int d = (e * LPR + lane) * VEC;
      if (v < V && d < D)
        hyb::store_v<VEC>(st + (long)v * D + d, S[r] + e * VEC);
    }
  }
}

namespace lin {

// Eight consecutive bf16 as floats, zero when !ok.
__device__ __forceinline__ void load8(const bf16 *p, bool ok, float *o) {
  uint4 v = make_uint4(0, 0, 0, 0);
  if (ok) v = *reinterpret_cast<const uint4 *>(p);
  unpack_bf16x2(v.x, o[0], o[1]);
  unpack_bf16x2(v.y, o[2], o[3]);
  unpack_bf16x2(v.z, o[4], o[5]);
  unpack_bf16x2(v.w, o[6], o[7]);
}

__device__ __forceinline__ void load8f(const float *p, bool ok, float *o) {
  float4 a = make_float4(0.f, 0.f, 0.f, 0.f), b = a;
  if (ok) {
    a = reinterpret_cast<const float4 *>(p)[0];
    b = reinterpret_cast<const float4 *>(p)[1];
  }
  o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w;
  o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
}

__device__ __forceinline__ bf16x8_t pack8(const float *v) {
  const uint4 u = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]),
                             pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
  return __builtin_bit_cast(bf16x8_t, u);
}

// (a, b) = hi + lo + O(2^-17): two packed bf16 pairs
__device__ __forceinline__ void split2(float a, float b, unsigned int &hi,
                                       unsigned int &lo) {
  hi = pack_bf16x2(a, b);
  lo = pack_bf16x2(a - __uint_as_float(hi << 16),
                   b - __uint_as_float(hi & 0xffff0000u));
}

__device__ __forceinline__ void split8(const float *v, bf16x8_t &hi,
                                       bf16x8_t &lo) {
  uint4 h, l;
  split2(v[0], v[1], h.x, l.x);
  split2(v[2], v[3], h.y, l.y);
  split2(v[4], v[5], h.z, l.z);
  split2(v[6], v[7], h.w, l.w);
  hi = __builtin_bit_cast(bf16x8_t, h);
  lo = __builtin_bit_cast(bf16x8_t, l);
}

// Eight activated elements, to be rounded to bf16 by the caller.
__device__ __forceinline__ void load8_act(const bf16 *p, bool ok, int act,
                                          float *o) {
  load8(p, ok, o);
  if (act != hyb::ACT_NONE) {
#pragma unroll
    for (int i = 0; i < 8; ++i) o[i] = hyb::activate<bf16>(o[i], act);
    if (!ok) {          // the activation of zero need not be zero
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = 0.f;
    }
  }
}

__device__ __forceinline__ float round_bf16(float v) { return bf2f(f2bf(v)); }

__device__ __forceinline__ f32x4_t mfma(const bf16x8_t &a, const bf16x8_t &b,
                                        const f32x4_t &c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

}  // namespace lin

// ---------------------------------------------------------------------------
// Own contribution of each chunk to the state at its end:
//   ws[chunk][h][v][d] = sum_j v_jv * (k_jd * decay from j to the end)
//   decay: CH ? log decay summed along the chunk [rows, H*D]
//             : powers of each head's decay [H][LIN_CHUNK + 1]
// A workgroup forms TD key channels x TV value channels.  A thread stages two
// neighbouring tokens at a time, so the [channel][token] images are written
// in dwords.
// Grid: (chunks, H, ceil(D/TD) * ceil(V/TV)); block 256.
// ---------------------------------------------------------------------------
template <bool CH, int TD, int TV>
__global__ void __launch_bounds__(256)
linear_chunk_state_kernel(float *__restrict__ ws,
                          const bf16 *__restrict__ proj, long stride,
                          int k_off, int v_off, int H, int D, int V, int act,
                          const float *__restrict__ decay,
                          const int *__restrict__ chunk_row0,
                          const int *__restrict__ chunk_len) {
  __shared__ __align__(16) bf16 v_s[TV * LIN_TS];
  __shared__ __align__(16) bf16 k_hi[TD * LIN_TS];
  __shared__ __align__(16) bf16 k_lo[TD * LIN_TS];
  const int chunk = blockIdx.x;
  const int h = blockIdx.y;
  const int nd = (D + TD - 1) / TD;
  const int d0 = (blockIdx.z % nd) * TD;
  const int v0 = (blockIdx.z / nd) * TV;
  const long row0 = chunk_row0[chunk];
  const int L = chunk_len[chunk];
  const int tid = threadIdx.x;
  const int wave = tid >> 6;
  const int lane = tid & 63;
  const int j = (tid & 31) * 2;               // tokens j, j + 1
  const int part = tid >> 5;                  // 8 channels of every 64
  const bf16 *p = proj + (row0 + j) * stride;
  const float *pw = decay + h * (LIN_CHUNK + 1);

#pragma unroll
  for (int c = part * 8; c < TD; c += 64) {
    float x[2][8];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const bool ok = j + u < L && d0 + c < D;
      lin::load8_act(p + u * stride + k_off + h * D + d0 + c, ok, act, x[u]);
      if constexpr (CH) {
        float end[8], cj[8];
        const long at = (row0 * H + h) * (long)D + d0 + c;
        lin::load8f(decay + at + (long)(L - 1) * H * D, ok, end);
        lin::load8f(decay + at + (long)(j + u) * H * D, ok, cj);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[u][e] *= __expf(end[e] - cj[e]);
      } else {
        const float w = ok ? pw[L - 1 - j - u] : 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) x[u][e] = lin::round_bf16(x[u][e]) * w;
      }
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      unsigned int hi, lo;
      lin::split2(x[0][e], x[1][e], hi, lo);
      *reinterpret_cast<unsigned int *>(k_hi + (c + e) * LIN_TS + j) = hi;
      *reinterpret_cast<unsigned int *>(k_lo + (c + e) * LIN_TS + j) = lo;
    }
  }
#pragma unroll
  for (int c = part * 8; c < TV; c += 64) {
    float x[2][8];
#pragma unroll
    for (int u = 0; u < 2; ++u)
      lin::load8_act(p + u * stride + v_off + h * V + v0 + c,
                     j + u < L && v0 + c < V, act, x[u]);
#pragma unroll
    for (int e = 0; e < 8; ++e)
      *reinterpret_cast<unsigned int *>(v_s + (c + e) * LIN_TS + j) =
          pack_bf16x2(x[0][e], x[1][e]);
  }
  __syncthreads();

  const int fr = lane & 15, g = lane >> 4;
  float *dst = ws + ((long)chunk * H + h) * (long)V * D;
#pragma unroll
  for (int vt = 0; vt < TV / 64; ++vt) {      // wave: 16 of every 64 values
    const int vr = vt * 64 + wave * 16;
    if (v0 + vr >= V) continue;               // wave-uniform
    bf16x8_t a[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
      a[kk] = *reinterpret_cast<const bf16x8_t *>(
          v_s + (vr + fr) * LIN_TS + kk * 32 + g * 8);
#pragma unroll
    for (int n = 0; n < TD / 16; ++n) {
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const int at = (n * 16 + fr) * LIN_TS + kk * 32 + g * 8;
        acc = lin::mfma(a[kk], *reinterpret_cast<const bf16x8_t *>(k_hi + at),
                        acc);
        acc = lin::mfma(a[kk], *reinterpret_cast<const bf16x8_t *>(k_lo + at),
                        acc);
      }
      const int d = d0 + n * 16 + fr;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int v = v0 + vr + g * 4 + r;
        if (v < V && d < D) dst[(long)v * D + d] = acc[r];
      }
    }
  }
}

// ---------------------------------------------------------------------------
// Scan along each sequence's chunks: ws[chunk] <- state at the chunk's start,
// as the operand the output kernel reads (every four floats become four bf16
// hi followed by their four bf16 lo, in place); the state after the last
// chunk goes to the pool in float32.  Four state elements per thread, loads
// of four chunks in flight.
// Grid: (sequences, H, ceil(V*D / 1024)); block 256.
// ---------------------------------------------------------------------------
template <bool CH>
__global__ void __launch_bounds__(256)
linear_chunk_scan_kernel(float *__restrict__ ws, float *__restrict__ state,
                         int H, int D, int V,
                         const float *__restrict__ decay,
                         const int *__restrict__ chunk_row0,
                         const int *__restrict__ chunk_len,
                         const int *__restrict__ seg_row0,
                         const int *__restrict__ seg_chunk0,
                         const int *__restrict__ seg_slot,
                         const int *__restrict__ positions) {
  const int seg = blockIdx.x;
  const int h = blockIdx.y;
  const int idx = (blockIdx.z * 256 + threadIdx.x) * 4;
  const int VD = V * D;
  if (idx >= VD) return;
  const int c0 = seg_chunk0[seg], c1 = seg_chunk0[seg + 1];
  if (c0 >= c1) return;
  const int d = idx % D;
  float *st = state + ((long)seg_slot[seg] * H + h) * (long)VD + idx;
  float S[4] = {0.f, 0.f, 0.f, 0.f};
  if (positions[seg_row0[seg]] != 0) hyb::load_v<4>(st, S);

  for (int cb = c0; cb < c1; cb += 4) {
    float own[4][4], dec[4][4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = cb + u;
      if (c < c1) {
        hyb::load_v<4>(ws + ((long)c * H + h) * (long)VD + idx, own[u]);
        const int len = chunk_len[c];
        if constexpr (CH) {
          hyb::load_v<4>(decay + (((long)chunk_row0[c] + len - 1) * H + h)
                                     * (long)D + d, dec[u]);
        } else {
          dec[u][0] = decay[h * (LIN_CHUNK + 1) + len];
        }
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = cb + u;
      if (c < c1) {
        uint4 out;
        lin::split2(S[0], S[1], out.x, out.z);
        lin::split2(S[2], S[3], out.y, out.w);
        *reinterpret_cast<uint4 *>(ws + ((long)c * H + h) * (long)VD + idx) =
            out;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float f = CH ? __expf(dec[u][i]) : dec[u][0];
          S[i] = f * S[i] + own[u][i];
        }
      }
    }
  }
  hyb::store_v<4>(st, S);
}

// ---------------------------------------------------------------------------
// Outputs of each chunk: o_i = qscale * (decayed q_i . S_start
//                                + sum_(j<=i) score(i, j) v_j).
// Four waves, wave w owns query rows 16w..16w+15.  Score tiles come out
// transposed (keys x queries), so a query's scores stay in one lane and
// become the A operand of the value product in registers.
//
// CH scores: with c the log decay summed from the chunk's start, the factor
// of channel d between i and j is exp(c_i - c_j), split at the end of the
// 16-row block before the wave's own rows: exp(c_i - c_ref), at most 1, times
// exp(c_ref - c_j), at most 1 for keys of earlier blocks.  For keys of the
// wave's own block the second factor is the inverse of the decay inside the
// block; where that could leave the float range (a channel that loses more
// than e^60 in 16 tokens) the block is formed pair by pair instead.
// Grid: (chunks, H); block 256.  NK = ceil(D/32).
// ---------------------------------------------------------------------------
template <bool CH, int NK>
__global__ void __launch_bounds__(256, CH ? (NK > 4 ? 2 : 3) : 4)
linear_chunk_out_kernel(bf16 *__restrict__ o, const float *__restrict__ ws,
                        const bf16 *__restrict__ proj, long stride, int q_off,
                        int k_off, int v_off, int H, int D, int V, int act,
                        float qscale, const float *__restrict__ decay,
                        const int *__restrict__ chunk_row0,
                        const int *__restrict__ chunk_len) {
  __shared__ __align__(16) bf16 v_s[64 * LIN_TS];
  const int chunk = blockIdx.x;
  const int h = blockIdx.y;
  const long row0 = chunk_row0[chunk];
  const int L = chunk_len[chunk];
  const int tid = threadIdx.x;
  const int wave = tid >> 6;
  const int lane = tid & 63;
  const int fr = lane & 15, g = lane >> 4;
  const int qi = wave * 16 + fr;               // this lane's query row
  const bool any = wave * 16 < L;              // this wave owns live rows
  const long HD = (long)H * D;
  const float *pw = decay + h * (LIN_CHUNK + 1);          // !CH
  const float *cum = decay + row0 * HD + (long)h * D;     // CH

  // query operand: plain for !CH; decayed from the chunk's start for CH
  bf16x8_t q_hi[NK], q_lo[CH ? NK : 1];
  f32x4_t s[4];
#pragma unroll
  for (int J = 0; J < 4; ++J) s[J] = (f32x4_t){0.f, 0.f, 0.f, 0.f};

  const bf16 *qp = proj + (row0 + min(qi, L - 1)) * stride + q_off + h * D;
  if constexpr (!CH) {
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const int d = kk * 32 + g * 8;
      float v[8];
      lin::load8_act(qp + d, qi < L && d < D, act, v);
      q_hi[kk] = lin::pack8(v);
    }
#pragma unroll
    for (int J = 0; J < 4; ++J) {
      if (J > wave || J * 16 >= L) continue;
      const int j = J * 16 + fr;
      const bf16 *kp = proj + (row0 + min(j, L - 1)) * stride + k_off + h * D;
#pragma unroll
      for (int kk = 0; kk < NK; ++kk) {
        const int d = kk * 32 + g * 8;
        float v[8];
        lin::load8_act(kp + d, j < L && d < D, act, v);
        s[J] = lin::mfma(lin::pack8(v), q_hi[kk], s[J]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = J * 16 + g * 4 + r;
        s[J][r] = (key <= qi && qi < L) ? s[J][r] * pw[qi - key] : 0.f;
      }
    }
  } else {
    const float *ci = cum + (long)min(qi, L - 1) * HD;
    const float *cref = cum + (long)(wave * 16 - 1) * HD;   // wave > 0
    const float *clast = cum + (long)min(wave * 16 + 15, L - 1) * HD;
    float drop = 0.f;                // most any channel loses in own block
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const int d = kk * 32 + g * 8;
      float ref[8], last[8];
      lin::load8f(cref + d, wave > 0 && any && d < D, ref);
      lin::load8f(clast + d, d < D, last);
#pragma unroll
      for (int e = 0; e < 8; ++e) drop = fmaxf(drop, ref[e] - last[e]);
    }
    const bool tame = !__any(any && drop > 60.f);           // wave-uniform
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const int d = kk * 32 + g * 8;
      const bool ok = qi < L && d < D;
      float q[8], c[8], x[8], ref[8];
      bf16x8_t a_hi, a_lo;
      lin::load8_act(qp + d, ok, act, q);
      lin::load8f(ci + d, ok, c);
      lin::load8f(cref + d, wave > 0 && any && d < D, ref);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = q[e] * __expf(c[e] - ref[e]);
      if (!ok) {
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = 0.f;
      }
      lin::split8(x, a_hi, a_lo);
      if (wave == 0) {                           // the start is the reference
        q_hi[kk] = a_hi;
        q_lo[kk] = a_lo;
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = q[e] * __expf(c[e]);
        lin::split8(x, q_hi[kk], q_lo[kk]);
      }
#pragma unroll
      for (int J = 0; J < 4; ++J) {
        if (J > wave || J * 16 >= L || (J == wave && !tame)) continue;
        const int j = J * 16 + fr;
        const bool k_ok = j < L && d < D;
        float k[8], cj[8];
        bf16x8_t b_hi, b_lo;
        lin::load8_act(proj + (row0 + min(j, L - 1)) * stride + k_off + h * D
                           + d, k_ok, act, k);
        lin::load8f(cum + (long)min(j, L - 1) * HD + d, k_ok, cj);
#pragma unroll
        for (int e = 0; e < 8; ++e) k[e] *= __expf(ref[e] - cj[e]);
        if (!k_ok) {
#pragma unroll
          for (int e = 0; e < 8; ++e) k[e] = 0.f;
        }
        lin::split8(k, b_hi, b_lo);
        s[J] = lin::mfma(b_hi, a_hi, s[J]);
        s[J] = lin::mfma(b_lo, a_hi, s[J]);
        s[J] = lin::mfma(b_hi, a_lo, s[J]);
      }
    }
    float dot[4] = {0.f, 0.f, 0.f, 0.f};
    if (!tame) {
      // own block, pair by pair: this lane's query against keys
      // wave*16 + g*4 + r
      for (int d = 0; d < D; d += 8) {
        float q[8], c[8];
        lin::load8_act(qp + d, true, act, q);
        lin::load8f(ci + d, true, c);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = min(wave * 16 + g * 4 + r, L - 1);
          float k[8], cj[8];
          lin::load8_act(proj + (row0 + j) * stride + k_off + h * D + d, true,
                         act, k);
          lin::load8f(cum + (long)j * HD + d, true, cj);
#pragma unroll
          for (int e = 0; e < 8; ++e)
            dot[r] = fmaf(q[e] * k[e], __expf(fminf(c[e] - cj[e], 0.f)),
                          dot[r]);
        }
      }
    }
#pragma unroll
    for (int J = 0; J < 4; ++J) {
      if (J != wave) continue;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = J * 16 + g * 4 + r;
        const float v = tame ? s[J][r] : dot[r];
        s[J][r] = (key <= qi && qi < L) ? v : 0.f;
      }
    }
  }

  bf16x8_t p_hi[2], p_lo[2];
#pragma unroll
  for (int kk = 0; kk < 2; ++kk) {
    p_hi[kk] = attn_core::scores_to_afrag(s[2 * kk], s[2 * kk + 1]);
    p_lo[kk] = attn_core::scores_to_afrag(attn_core::bf16_rest(s[2 * kk]),
                                          attn_core::bf16_rest(s[2 * kk + 1]));
  }

  const float *S = ws + ((long)chunk * H + h) * (long)V * D;
  for (int v0 = 0; v0 < V; v0 += 64) {
    if (v0) __syncthreads();
    {
      const int j = (tid & 31) * 2;            // tokens j, j + 1
      const int c = (tid >> 5) * 8;
      float x[2][8];
#pragma unroll
      for (int u = 0; u < 2; ++u)
        lin::load8_act(proj + (row0 + min(j + u, L - 1)) * stride + v_off
                           + h * V + v0 + c, j + u < L && v0 + c < V, act,
                       x[u]);
#pragma unroll
      for (int e = 0; e < 8; ++e)
        *reinterpret_cast<unsigned int *>(v_s + (c + e) * LIN_TS + j) =
            pack_bf16x2(x[0][e], x[1][e]);
    }
    __syncthreads();
#pragma unroll
    for (int vt = 0; vt < 4; ++vt) {
      const int vb = v0 + vt * 16;
      if (vb >= V || !any) continue;           // wave-uniform
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NK; ++kk) {
        const int d = kk * 32 + g * 8;
        uint4 x = make_uint4(0, 0, 0, 0), y = x;
        if (vb + fr < V && d < D) {
          const uint4 *at = reinterpret_cast<const uint4 *>(
              S + (long)(vb + fr) * D + d);
          x = at[0];
          y = at[1];
        }
        const bf16x8_t s_hi = __builtin_bit_cast(
            bf16x8_t, make_uint4(x.x, x.y, y.x, y.y));
        const bf16x8_t s_lo = __builtin_bit_cast(
            bf16x8_t, make_uint4(x.z, x.w, y.z, y.w));
        acc = lin::mfma(q_hi[kk], s_hi, acc);
        acc = lin::mfma(q_hi[kk], s_lo, acc);
        if constexpr (CH) acc = lin::mfma(q_lo[kk], s_hi, acc);
      }
      if constexpr (!CH) {
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[r] *= pw[wave * 16 + g * 4 + r + 1];
      }
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const bf16x8_t b = *reinterpret_cast<const bf16x8_t *>(
            v_s + (vt * 16 + fr) * LIN_TS + kk * 32 + g * 8);
        acc = lin::mfma(p_hi[kk], b, acc);
        acc = lin::mfma(p_lo[kk], b, acc);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = wave * 16 + g * 4 + r;
        if (i < L && vb + fr < V)
          o[((row0 + i) * H + h) * (long)V + vb + fr] = f2bf(acc[r] * qscale);
      }
    }
  }
}
