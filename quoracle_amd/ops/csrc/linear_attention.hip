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
          q[e * VEC + i] = hyb::activate(q[e * VEC + i], act);
          k[e * VEC + i] = hyb::activate(k[e * VEC + i], act);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
      const int vi = v_base + r * RPG;
      v[r] = vi < V ? hyb::activate(hyb::to_f(p[v_off + h * V + vi]), act)
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

// v = hi + lo + O(2^-17 v)
__device__ __forceinline__ void split8(const float *v, bf16x8_t &hi,
                                       bf16x8_t &lo) {
  float r[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) r[i] = v[i] - bf2f(f2bf(v[i]));
  hi = pack8(v);
  lo = pack8(r);
}

// Eight activated elements, rounded to bf16 (the tiles' input precision).
__device__ __forceinline__ void load8_act(const bf16 *p, bool ok, int act,
                                          float *o) {
  load8(p, ok, o);
  if (act != hyb::ACT_NONE) {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      o[i] = ok ? bf2f(f2bf(hyb::activate(o[i], act))) : 0.f;
  }
}

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
// Grid: (chunks, H, ceil(D/64) * ceil(V/64)); block 256.
// ---------------------------------------------------------------------------
template <bool CH>
__global__ void __launch_bounds__(256)
linear_chunk_state_kernel(float *__restrict__ ws,
                          const bf16 *__restrict__ proj, long stride,
                          int k_off, int v_off, int H, int D, int V, int act,
                          const float *__restrict__ decay,
                          const int *__restrict__ chunk_row0,
                          const int *__restrict__ chunk_len) {
  __shared__ __align__(16) bf16 v_s[64 * LIN_TS];
  __shared__ __align__(16) bf16 k_hi[64 * LIN_TS];
  __shared__ __align__(16) bf16 k_lo[64 * LIN_TS];
  const int chunk = blockIdx.x;
  const int h = blockIdx.y;
  const int nd = (D + 63) / 64;
  const int d0 = (blockIdx.z % nd) * 64;
  const int v0 = (blockIdx.z / nd) * 64;
  const long row0 = chunk_row0[chunk];
  const int L = chunk_len[chunk];
  const int tid = threadIdx.x;
  const int j = tid & 63;
  const int wave = tid >> 6;
  const int lane = tid & 63;
  const bool live = j < L;
  const bf16 *p = proj + (row0 + j) * stride;
  const float w_head = CH ? 0.f
      : decay[h * (LIN_CHUNK + 1) + (live ? L - 1 - j : 0)];

#pragma unroll
  for (int half = 0; half < 2; ++half) {
    const int c = wave * 16 + half * 8;
    float kv[8], w[8];
    const bool k_ok = live && d0 + c < D;
    lin::load8_act(p + k_off + h * D + d0 + c, k_ok, act, kv);
    if constexpr (CH) {
      float end[8];
      const long at = (row0 * H + h) * (long)D + d0 + c;
      lin::load8f(decay + at + (long)(L - 1) * H * D, k_ok, end);
      lin::load8f(decay + at + (long)j * H * D, k_ok, w);
#pragma unroll
      for (int e = 0; e < 8; ++e) w[e] = expf(end[e] - w[e]);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) w[e] = w_head;
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float x = kv[e] * w[e];
      const bf16 hi = f2bf(x);
      k_hi[(c + e) * LIN_TS + j] = hi;
      k_lo[(c + e) * LIN_TS + j] = f2bf(x - bf2f(hi));
    }
    float vv[8];
    lin::load8_act(p + v_off + h * V + v0 + c, live && v0 + c < V, act, vv);
#pragma unroll
    for (int e = 0; e < 8; ++e) v_s[(c + e) * LIN_TS + j] = f2bf(vv[e]);
  }
  __syncthreads();

  const int fr = lane & 15, g = lane >> 4;
  f32x4_t acc[4];
#pragma unroll
  for (int n = 0; n < 4; ++n) acc[n] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int kk = 0; kk < 2; ++kk) {
    const int jo = kk * 32 + g * 8;
    const bf16x8_t a = *reinterpret_cast<const bf16x8_t *>(
        v_s + (wave * 16 + fr) * LIN_TS + jo);
#pragma unroll
    for (int n = 0; n < 4; ++n) {
      acc[n] = lin::mfma(a, *reinterpret_cast<const bf16x8_t *>(
          k_hi + (n * 16 + fr) * LIN_TS + jo), acc[n]);
      acc[n] = lin::mfma(a, *reinterpret_cast<const bf16x8_t *>(
          k_lo + (n * 16 + fr) * LIN_TS + jo), acc[n]);
    }
  }
  float *dst = ws + ((long)chunk * H + h) * (long)V * D;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int v = v0 + wave * 16 + g * 4 + r;
    if (v >= V) continue;
#pragma unroll
    for (int n = 0; n < 4; ++n) {
      const int d = d0 + n * 16 + fr;
      if (d < D) dst[(long)v * D + d] = acc[n][r];
    }
  }
}

// ---------------------------------------------------------------------------
// Scan along each sequence's chunks: ws[chunk] <- state at the chunk's start;
// the state after the last chunk goes to the pool.  Four state elements per
// thread, loads of four chunks in flight.
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
        hyb::store_v<4>(ws + ((long)c * H + h) * (long)VD + idx, S);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float f = CH ? expf(dec[u][i]) : dec[u][0];
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
// of channel d between i and j is exp(c_i - c_j).  Against the keys of an
// earlier 16-row block it is split at the end of the block before the
// wave's own rows, exp(c_i - c_ref) * exp(c_ref - c_j), both at most 1; in
// the wave's own block it is formed pair by pair.  No factor can overflow,
// whatever the decay.
// Grid: (chunks, H); block 256.  NK = ceil(D/32).
// ---------------------------------------------------------------------------
template <bool CH, int NK>
__global__ void __launch_bounds__(256)
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
  const long HD = (long)H * D;
  const float *pw = decay + h * (LIN_CHUNK + 1);          // !CH
  const float *cum = decay + row0 * HD + (long)h * D;     // CH

  // query operand(s): plain for !CH; decayed from the chunk's start for CH
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
    const bool any = wave * 16 < L;              // this wave owns live rows
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) {
      const int d = kk * 32 + g * 8;
      const bool ok = any && qi < L && d < D;
      float q[8], c[8], x[8], ref[8];
      lin::load8_act(qp + d, ok, act, q);
      lin::load8f(ci + d, ok, c);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = q[e] * expf(c[e]);
      lin::split8(x, q_hi[kk], q_lo[kk]);
      if (any && wave > 0) {                     // wave-uniform
        bf16x8_t a_hi, a_lo;
        lin::load8f(cref + d, d < D, ref);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = ok ? q[e] * expf(c[e] - ref[e])
                                              : 0.f;
        lin::split8(x, a_hi, a_lo);
#pragma unroll
        for (int J = 0; J < 3; ++J) {
          if (J >= wave) continue;
          const int j = J * 16 + fr;             // < wave*16 <= L
          float k[8], cj[8];
          bf16x8_t b_hi, b_lo;
          lin::load8_act(proj + (row0 + j) * stride + k_off + h * D + d,
                         d < D, act, k);
          lin::load8f(cum + (long)j * HD + d, d < D, cj);
#pragma unroll
          for (int e = 0; e < 8; ++e) k[e] *= expf(ref[e] - cj[e]);
          lin::split8(k, b_hi, b_lo);
          s[J] = lin::mfma(b_hi, a_hi, s[J]);
          s[J] = lin::mfma(b_lo, a_hi, s[J]);
          s[J] = lin::mfma(b_hi, a_lo, s[J]);
        }
      }
    }
    // own block, pair by pair in float32: this lane's query against keys
    // wave*16 + g*4 + r
    if (any) {
      float dot[4] = {0.f, 0.f, 0.f, 0.f};
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
#pragma unroll
      for (int J = 0; J < 4; ++J) {
        if (J != wave) continue;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = J * 16 + g * 4 + r;
          s[J][r] = (key <= qi && qi < L) ? dot[r] : 0.f;
        }
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
      const int j = tid & 63;
      const bf16 *vp = proj + (row0 + min(j, L - 1)) * stride + v_off + h * V;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const int c = wave * 16 + half * 8;
        float vv[8];
        lin::load8_act(vp + v0 + c, j < L && v0 + c < V, act, vv);
#pragma unroll
        for (int e = 0; e < 8; ++e) v_s[(c + e) * LIN_TS + j] = f2bf(vv[e]);
      }
    }
    __syncthreads();
#pragma unroll
    for (int vt = 0; vt < 4; ++vt) {
      const int vb = v0 + vt * 16;
      if (vb >= V || wave * 16 >= L) continue;   // wave-uniform
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NK; ++kk) {
        const int d = kk * 32 + g * 8;
        float x[8];
        bf16x8_t s_hi, s_lo;
        lin::load8f(S + (long)(vb + fr) * D + d, vb + fr < V && d < D, x);
        lin::split8(x, s_hi, s_lo);
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
