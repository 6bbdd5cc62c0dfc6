// Paged attention confined to position chunks, with an optional sink that
// adds one to the softmax denominator (gfx950).
//
//   * bf16, head dimension a multiple of 8 up to 128: the matrix-core
//     prefill tile and flash-decode of attention_core.h (LOCAL form).
//   * any other head dimension, and float32: one workgroup per (query row,
//     head) on the vector ALU.
//
// KV cache layout as everywhere: [num_blocks, Hkv, BLOCK_SIZE, D].

#include "attention_core.h"
#include "hybrid_common.h"

template <int DP>
__global__ void __launch_bounds__(512, 4)
local_attn_prefill_kernel(
    bf16 *__restrict__ out, float *__restrict__ part_m,
    float *__restrict__ part_l, float *__restrict__ part_acc,
    const bf16 *__restrict__ q, const bf16 *__restrict__ kc,
    const bf16 *__restrict__ vc, const int *__restrict__ bt,
    const int *__restrict__ tile_q0, const int *__restrict__ tile_qn,
    const int *__restrict__ tile_seq, const int *__restrict__ tile_pos0,
    float scale, int Hq, int Hkv, int BS, int MAXB, int GQ, int NS, int D,
    int chunk, bool sink) {
  attn_core::prefill_t12<DP, true>(out, part_m, part_l, part_acc, q, kc, vc,
                                   bt, tile_q0, tile_qn, tile_seq, tile_pos0,
                                   scale, Hq, Hkv, BS, MAXB, GQ, NS, D, chunk,
                                   sink);
}

template <int DP>
__global__ void __launch_bounds__(256)
local_attn_decode_kernel(
    float *__restrict__ part_m, float *__restrict__ part_l,
    float *__restrict__ part_acc, const bf16 *__restrict__ q,
    const bf16 *__restrict__ kc, const bf16 *__restrict__ vc,
    const int *__restrict__ bt, const int *__restrict__ ctx, float scale,
    int Hq, int Hkv, int BS, int MAXB, int GQ, int NS, int D, int chunk,
    bool sink) {
  attn_core::decode_mfma<DP, true>(part_m, part_l, part_acc, q, kc, vc, bt,
                                   ctx, scale, Hq, Hkv, BS, MAXB, GQ, NS, D,
                                   chunk, sink);
}

// Grid: (B, Hq); block 128.
__global__ void __launch_bounds__(128)
local_attn_decode_combine_kernel(bf16 *__restrict__ out,
                                 const float *__restrict__ part_m,
                                 const float *__restrict__ part_l,
                                 const float *__restrict__ part_acc, int Hq,
                                 int D, int NS) {
  const long row = (long)blockIdx.x * Hq + blockIdx.y;
  attn_core::combine_splits(out + row * D, part_m, part_l, part_acc, row * NS,
                            1, D, NS);
}

// Grid: (tiles, Hq, 128); block 128.
__global__ void __launch_bounds__(128)
local_attn_prefill_combine_kernel(bf16 *__restrict__ out,
                                  const float *__restrict__ part_m,
                                  const float *__restrict__ part_l,
                                  const float *__restrict__ part_acc,
                                  const int *__restrict__ tile_q0,
                                  const int *__restrict__ tile_qn, int Hq,
                                  int D, int NS) {
  const int tile = blockIdx.x;
  const int h = blockIdx.y;
  const int qi = blockIdx.z;
  if (qi >= tile_qn[tile]) return;
  const long row = (long)(tile_q0[tile] + qi) * Hq + h;
  attn_core::combine_splits(out + row * D, part_m, part_l, part_acc,
                            (((long)tile * Hq + h) * NS) * 128 + qi, 128, D,
                            NS);
}

// ---------------------------------------------------------------------------
// Vector-ALU form: any head dimension, bf16 or float32.  Row r belongs to
// sequence row_seq[r] and sits at position row_pos[r].
// Grid: (rows, Hq); block 128; dynamic LDS 2*D floats.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void __launch_bounds__(128)
local_attn_rows_kernel(T *__restrict__ out, const T *__restrict__ q,
                       const T *__restrict__ kc, const T *__restrict__ vc,
                       const int *__restrict__ bt,
                       const int *__restrict__ row_seq,
                       const int *__restrict__ row_pos, float scale, int Hq,
                       int Hkv, int D, int BS, int MAXB, int GQ, int chunk,
                       bool sink) {
  extern __shared__ float dyn_s[];
  float *q_s = dyn_s;
  float *acc_s = dyn_s + D;
  __shared__ float p_s[128];
  __shared__ long base_s[128];
  __shared__ float scratch[2];
  const long row = blockIdx.x;
  const int h = blockIdx.y;
  const int hk = h / GQ;
  const int tid = threadIdx.x;
  const int pos = row_pos[row];
  const int seq = row_seq[row];
  const int low = chunk > 0 ? pos / chunk * chunk : 0;

  for (int d = tid; d < D; d += 128) {
    q_s[d] = hyb::to_f(q[(row * Hq + h) * (long)D + d]);
    acc_s[d] = 0.f;
  }
  __syncthreads();

  float m = sink ? 0.f : -INFINITY;
  float l = sink ? 1.f : 0.f;
  for (int start = low; start <= pos; start += 128) {
    const int n = min(128, pos + 1 - start);
    float s = -INFINITY;
    if (tid < n) {
      const int token = start + tid;
      const long blk = bt[(long)seq * MAXB + token / BS];
      const long base = ((blk * Hkv + hk) * BS + token % BS) * (long)D;
      base_s[tid] = base;
      float dot = 0.f;
      for (int d = 0; d < D; ++d)
        dot = fmaf(q_s[d], hyb::to_f(kc[base + d]), dot);
      s = dot * scale;
    }
    const float mn = fmaxf(m, block_max(s, scratch));
    const float alpha = (m == -INFINITY) ? 0.f : expf(m - mn);
    const float p = tid < n ? expf(s - mn) : 0.f;
    p_s[tid] = p;
    l = l * alpha + block_sum(p, scratch);   // its barriers publish p_s
    m = mn;
    for (int d = tid; d < D; d += 128) {
      float a = acc_s[d] * alpha;
      for (int t = 0; t < n; ++t)
        a = fmaf(p_s[t], hyb::to_f(vc[base_s[t] + d]), a);
      acc_s[d] = a;
    }
    __syncthreads();
  }
  for (int d = tid; d < D; d += 128)
    hyb::put(out + (row * Hq + h) * (long)D + d, acc_s[d] / l);
}
