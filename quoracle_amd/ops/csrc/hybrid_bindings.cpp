// Torch bindings of the hybrid-model kernels (gfx950): chunk-local attention
// with a sink, linear attention with a decaying state, and the norms and
// gates around them, for bf16 and float32 activations.  One translation unit,
// built in-tree by quoracle_amd/ops/build.py.

#include <torch/extension.h>

#include <c10/hip/HIPStream.h>

#include <stdexcept>
#include <string>

#include "stream_kernels.hip"
#include "attention_local.hip"
#include "linear_attention.hip"
#include "hybrid_elementwise.hip"

namespace {

#include "hybrid_host.h"

void post_norm(Tensor x, Tensor h, Tensor a, double sa, OptTensor b,
               double sb, double alpha, Tensor w, double eps) {
  CHECK_F32(x); CHECK_GPU(h); CHECK_GPU(a); CHECK_F32(w);
  const int n = w.size(0);
  const long T = x.numel() / n;
  TORCH_CHECK(x.numel() == T * n && h.numel() == T * n && a.numel() == T * n,
              "post_norm shapes");
  if (b) { CHECK_GPU(*b); TORCH_CHECK(b->numel() == T * n, "post_norm b"); }
  if (T == 0) return;
  by_dtype(h, [&](auto t0) {
    using A = decltype(t0);
    by_vec(n % 8 == 0, [&](auto v) {
      by_items(n, v, [&](auto ni) {
        post_norm_kernel<A, decltype(v)::value, decltype(ni)::value>
            <<<dim3(T), dim3(256), 0, current_stream()>>>(
                fptr(x), ptr<A>(h), ptr<A>(a), (float)sa,
                b ? ptr<A>(*b) : nullptr, (float)sb, (float)alpha, fptr(w), n,
                (float)eps);
      });
    });
  });
  HIP_CHECK_KERNEL();
}

void glu(Tensor out, Tensor gu) {
  CHECK_GPU(out); CHECK_GPU(gu);
  const int n = out.size(-1);
  const long T = out.numel() / n;
  TORCH_CHECK(gu.numel() == T * 2 * n, "glu shapes");
  if (T == 0) return;
  by_dtype(out, [&](auto t0) {
    using A = decltype(t0);
    by_vec(n % 8 == 0, [&](auto v) {
      constexpr int VEC = decltype(v)::value;
      glu_kernel<A, VEC>
          <<<dim3(T, (n + 256 * VEC - 1) / (256 * VEC)), dim3(256), 0,
             current_stream()>>>(ptr<A>(out), ptr<A>(gu), n);
    });
  });
  HIP_CHECK_KERNEL();
}

void gated_norm(Tensor out, Tensor o, Tensor proj, int64_t g_off, Tensor w,
                int64_t groups, int64_t act, double eps) {
  CHECK_GPU(out); CHECK_GPU(o); CHECK_GPU(proj); CHECK_F32(w);
  const int n = w.size(0);
  const long T = proj.size(0), stride = proj.size(1);
  TORCH_CHECK(o.numel() == T * groups * n && out.numel() == o.numel(),
              "gated_norm shapes");
  TORCH_CHECK(g_off + groups * n <= stride, "gated_norm gate");
  if (T == 0) return;
  const bool vec = n % 8 == 0 && stride % 8 == 0 && g_off % 8 == 0;
  by_dtype(out, [&](auto t0) {
    using A = decltype(t0);
    by_vec(vec, [&](auto v) {
      constexpr int VEC = decltype(v)::value;
      auto small = [&](auto lpg) {
        constexpr int LPG = decltype(lpg)::value;
        gated_norm_small_kernel<A, VEC, LPG>
            <<<dim3((T * groups * LPG + 255) / 256), dim3(256), 0,
               current_stream()>>>(
                ptr<A>(out), ptr<A>(o), ptr<A>(proj), stride, (int)g_off,
                fptr(w), n, (int)groups, T * groups, (int)act, (float)eps);
      };
      if (n <= 8 * VEC) small(Int<8>());
      else if (n <= 16 * VEC) small(Int<16>());
      else if (n <= 64 * VEC) small(Int<64>());
      else
        by_items(n, v, [&](auto ni) {
          gated_norm_kernel<A, VEC, decltype(ni)::value>
              <<<dim3(T, groups), dim3(256), 0, current_stream()>>>(
                  ptr<A>(out), ptr<A>(o), ptr<A>(proj), stride, (int)g_off,
                  fptr(w), n, (int)act, (float)eps);
        });
    });
  });
  HIP_CHECK_KERNEL();
}

void qk_norm_rope_store(Tensor q_out, Tensor kcache, Tensor vcache,
                        Tensor proj, int64_t q_off, int64_t k_off, Tensor qw,
                        Tensor kw, Tensor positions, Tensor slots,
                        Tensor freq, double mag, double eps) {
  CHECK_GPU(q_out); CHECK_GPU(kcache); CHECK_GPU(vcache); CHECK_GPU(proj);
  CHECK_F32(qw); CHECK_F32(kw); CHECK_I32(positions); CHECK_I32(slots);
  CHECK_GPU(freq);
  TORCH_CHECK(freq.scalar_type() == torch::kFloat64, "freq must be float64");
  const long T = proj.size(0), stride = proj.size(1);
  const int H = q_out.size(1), D = q_out.size(2);
  const int G = kcache.size(1), BS = kcache.size(2);
  const int pairs = freq.size(0);
  TORCH_CHECK(q_out.size(0) == T && kcache.size(3) == D &&
              vcache.sizes() == kcache.sizes(), "qk_norm_rope_store cache");
  TORCH_CHECK(qw.numel() == (long)H * D && kw.numel() == (long)G * D &&
              2 * pairs <= D && pairs <= 2048, "qk_norm_rope_store sizes");
  TORCH_CHECK(q_off + H * D <= stride && k_off + G * D <= stride,
              "qk_norm_rope_store offsets");
  TORCH_CHECK(positions.size(0) == T && slots.size(0) == T, "rows");
  if (T == 0) return;
  by_dtype(q_out, [&](auto t0) {
    using A = decltype(t0);
    auto run = [&](auto kernel) {
      kernel<<<dim3(T), dim3(256), 2 * pairs * sizeof(float),
               current_stream()>>>(
          ptr<A>(q_out), ptr<A>(kcache), ptr<A>(vcache), ptr<A>(proj), stride,
          (int)q_off, (int)k_off, fptr(qw), fptr(kw), iptr(positions),
          iptr(slots), freq.data_ptr<double>(), pairs, (float)mag, (float)eps,
          H, G, D, BS);
    };
    const long groups = (long)(H + G) * D / 8;
    if (D % 8 || stride % 8 || q_off % 8 || k_off % 8 || groups > 4 * 256)
      run(qk_norm_rope_store_kernel<A>);
    else if (groups <= 256) run(qk_norm_rope_store8_kernel<A, 1>);
    else if (groups <= 512) run(qk_norm_rope_store8_kernel<A, 2>);
    else run(qk_norm_rope_store8_kernel<A, 4>);
  });
  HIP_CHECK_KERNEL();
}

// Rows [first, first + rows) as runs; run arrays null: one run per row.
void log_decay(Tensor out, Tensor proj, int64_t a_off, Tensor a2, Tensor bias,
               double tau, int64_t first, int64_t rows, OptTensor run_row0,
               OptTensor run_len) {
  CHECK_F32(out); CHECK_GPU(proj); CHECK_GPU(a2); CHECK_F32(bias);
  const int C = a2.size(0), rank = a2.size(1);
  const long stride = proj.size(1);
  TORCH_CHECK(out.size(0) == proj.size(0) && out.numel() == out.size(0) * C &&
              bias.numel() == C && a_off + rank <= stride &&
              first + rows <= proj.size(0), "log_decay shapes");
  long runs = rows;
  if (run_row0) {
    CHECK_I32(*run_row0); CHECK_I32(*run_len);
    runs = run_row0->size(0);
    first = 0;                                  // run rows are absolute
  }
  if (runs == 0) return;
  by_dtype(proj, [&](auto t0) {
    using A = decltype(t0);
    auto run = [&](auto rmax) {
      log_decay_kernel<A, decltype(rmax)::value>
          <<<dim3(runs, (C + 63) / 64), dim3(256), 0, current_stream()>>>(
              fptr(out) + first * C, ptr<A>(proj) + first * stride, stride,
              (int)a_off, rank, ptr<A>(a2), fptr(bias), (float)(1.0 / tau),
              C, run_row0 ? iptr(*run_row0) : nullptr,
              run_row0 ? iptr(*run_len) : nullptr);
    };
    if (rank <= 16) run(Int<16>());
    else if (rank <= 64) run(Int<64>());
    else run(Int<0>());
  });
  HIP_CHECK_KERNEL();
}

// -- attention ---------------------------------------------------------------

struct AttnDims {
  int Hq, Hkv, D, BS, MAXB, GQ;
};

AttnDims attn_dims(const Tensor &q, const Tensor &kc, const Tensor &vc,
                   const Tensor &bt) {
  CHECK_GPU(q); CHECK_GPU(kc); CHECK_GPU(vc); CHECK_I32(bt);
  AttnDims a{(int)q.size(1), (int)kc.size(1), (int)q.size(2),
             (int)kc.size(2), (int)bt.size(1), 0};
  TORCH_CHECK(kc.size(3) == a.D && vc.sizes() == kc.sizes() &&
              a.Hq % a.Hkv == 0, "attention shapes");
  a.GQ = a.Hq / a.Hkv;
  return a;
}

bool attn_tiles_ok(const Tensor &q) {
  return q.scalar_type() == torch::kBFloat16 && q.size(2) <= 128 &&
         q.size(2) % 8 == 0;
}

void local_attn_rows(Tensor out, Tensor q, Tensor kc, Tensor vc, Tensor bt,
                     Tensor row_seq, Tensor row_pos, double scale,
                     int64_t chunk, bool sink) {
  const AttnDims a = attn_dims(q, kc, vc, bt);
  CHECK_GPU(out); CHECK_I32(row_seq); CHECK_I32(row_pos);
  const long T = row_seq.size(0);
  TORCH_CHECK(q.size(0) >= T && out.size(0) >= T && row_pos.size(0) >= T &&
              a.D <= 4096, "local_attn_rows shapes");
  if (T == 0) return;
  by_dtype(q, [&](auto t0) {
    using A = decltype(t0);
    local_attn_rows_kernel<A>
        <<<dim3(T, a.Hq), dim3(128), 2 * a.D * sizeof(float),
           current_stream()>>>(
            ptr<A>(out), ptr<A>(q), ptr<A>(kc), ptr<A>(vc), iptr(bt),
            iptr(row_seq), iptr(row_pos), (float)scale, a.Hq, a.Hkv, a.D,
            a.BS, a.MAXB, a.GQ, (int)chunk, sink);
  });
  HIP_CHECK_KERNEL();
}

// Tiles of at most 128 query rows; max_kv bounds the keys any tile sees.
void local_attn_prefill(Tensor out, Tensor q, Tensor kc, Tensor vc, Tensor bt,
                        Tensor tile_q0, Tensor tile_qn, Tensor tile_seq,
                        Tensor tile_pos0, double scale, int64_t chunk,
                        bool sink, int64_t max_kv) {
  const AttnDims a = attn_dims(q, kc, vc, bt);
  CHECK_GPU(out); CHECK_I32(tile_q0); CHECK_I32(tile_qn);
  CHECK_I32(tile_seq); CHECK_I32(tile_pos0);
  TORCH_CHECK(attn_tiles_ok(q), "local_attn_prefill: dtype or head dim");
  const long nt = tile_q0.size(0);
  if (nt == 0) return;
  long seen = max_kv;
  if (chunk > 0) seen = std::min<long>(seen, chunk + 127);
  long ns = 1;
  if (seen >= 1024)
    ns = std::max<long>(1, std::min<long>({16, 512 / (nt * a.Hq),
                                           seen / 256}));
  Tensor pm, pl, pa;
  if (ns > 1) {
    auto opts = q.options().dtype(torch::kFloat32);
    pm = torch::empty({nt, a.Hq, ns, 128}, opts);
    pl = torch::empty({nt, a.Hq, ns, 128}, opts);
    pa = torch::empty({nt, a.Hq, ns, 128, a.D}, opts);
  }
  auto run = [&](auto dp) {
    local_attn_prefill_kernel<decltype(dp)::value>
        <<<dim3(nt, a.Hq, ns), dim3(512), 0, current_stream()>>>(
            ptr<bf16>(out), ns > 1 ? fptr(pm) : nullptr,
            ns > 1 ? fptr(pl) : nullptr, ns > 1 ? fptr(pa) : nullptr,
            ptr<bf16>(q), ptr<bf16>(kc), ptr<bf16>(vc), iptr(bt),
            iptr(tile_q0), iptr(tile_qn), iptr(tile_seq), iptr(tile_pos0),
            (float)scale, a.Hq, a.Hkv, a.BS, a.MAXB, a.GQ, (int)ns, a.D,
            (int)chunk, sink);
  };
  if (a.D <= 64) run(std::integral_constant<int, 64>());
  else run(std::integral_constant<int, 128>());
  HIP_CHECK_KERNEL();
  if (ns > 1) {
    local_attn_prefill_combine_kernel
        <<<dim3(nt, a.Hq, 128), dim3(128), 0, current_stream()>>>(
            ptr<bf16>(out), fptr(pm), fptr(pl), fptr(pa), iptr(tile_q0),
            iptr(tile_qn), a.Hq, a.D, (int)ns);
    HIP_CHECK_KERNEL();
  }
}

// One query row per sequence; max_ctx bounds ctx_lens.
void local_attn_decode(Tensor out, Tensor q, Tensor kc, Tensor vc, Tensor bt,
                       Tensor ctx_lens, double scale, int64_t chunk,
                       bool sink, int64_t max_ctx) {
  const AttnDims a = attn_dims(q, kc, vc, bt);
  CHECK_GPU(out); CHECK_I32(ctx_lens);
  TORCH_CHECK(attn_tiles_ok(q) && a.GQ <= 16,
              "local_attn_decode: dtype, head dim or group size");
  const long B = ctx_lens.size(0);
  TORCH_CHECK(q.size(0) >= B && out.size(0) >= B && bt.size(0) >= B, "rows");
  if (B == 0) return;
  long seen = max_ctx;
  if (chunk > 0) seen = std::min<long>(seen, chunk);
  const long ns = std::max<long>(1, std::min<long>(32, seen / 256));
  auto opts = q.options().dtype(torch::kFloat32);
  auto pm = torch::empty({B, a.Hq, ns}, opts);
  auto pl = torch::empty({B, a.Hq, ns}, opts);
  auto pa = torch::empty({B, a.Hq, ns, a.D}, opts);
  auto run = [&](auto dp) {
    local_attn_decode_kernel<decltype(dp)::value>
        <<<dim3(B, a.Hkv, ns), dim3(256), 0, current_stream()>>>(
            fptr(pm), fptr(pl), fptr(pa), ptr<bf16>(q), ptr<bf16>(kc),
            ptr<bf16>(vc), iptr(bt), iptr(ctx_lens), (float)scale, a.Hq,
            a.Hkv, a.BS, a.MAXB, a.GQ, (int)ns, a.D, (int)chunk, sink);
  };
  if (a.D <= 64) run(std::integral_constant<int, 64>());
  else run(std::integral_constant<int, 128>());
  HIP_CHECK_KERNEL();
  local_attn_decode_combine_kernel
      <<<dim3(B, a.Hq), dim3(128), 0, current_stream()>>>(
          ptr<bf16>(out), fptr(pm), fptr(pl), fptr(pa), a.Hq, a.D, (int)ns);
  HIP_CHECK_KERNEL();
}

// -- linear attention --------------------------------------------------------

struct LinDims {
  long stride;
  int q_off, k_off, v_off, H, D, V;
};

LinDims lin_dims(const Tensor &o, const Tensor &proj, const Tensor &state,
                 int64_t q_off, int64_t k_off, int64_t v_off) {
  CHECK_GPU(o); CHECK_GPU(proj); CHECK_F32(state);
  TORCH_CHECK(state.dim() == 4, "state must be [slots, H, V, D]");
  LinDims a{proj.size(1), (int)q_off, (int)k_off, (int)v_off,
            (int)state.size(1), (int)state.size(3), (int)state.size(2)};
  TORCH_CHECK(o.size(0) == proj.size(0) &&
              o.numel() == proj.size(0) * a.H * a.V, "linear output shape");
  TORCH_CHECK(q_off + a.H * a.D <= a.stride && k_off + a.H * a.D <= a.stride &&
              v_off + a.H * a.V <= a.stride, "linear projection offsets");
  TORCH_CHECK(a.D <= 512, "linear attention key dim above 512");
  return a;
}

void check_decay(const Tensor &decay, const LinDims &a, long rows,
                 bool channel, long per_head) {
  CHECK_F32(decay);
  TORCH_CHECK(decay.numel() == (channel ? rows * a.H * a.D : a.H * per_head),
              "decay shape");
}

// seg_row0 null: rows 0..B-1 are one-token sequences with slots seg_slot.
void linear_recurrent(Tensor o, Tensor proj, int64_t q_off, int64_t k_off,
                      int64_t v_off, int64_t act, double qscale, Tensor decay,
                      bool channel, Tensor state, OptTensor seg_row0,
                      OptTensor seg_len, Tensor seg_slot, Tensor positions) {
  const LinDims a = lin_dims(o, proj, state, q_off, k_off, v_off);
  check_decay(decay, a, proj.size(0), channel, 1);
  CHECK_I32(seg_slot); CHECK_I32(positions);
  if (seg_row0) {
    CHECK_I32(*seg_row0); CHECK_I32(*seg_len);
    TORCH_CHECK(seg_row0->size(0) == seg_slot.size(0) &&
                seg_len->size(0) == seg_slot.size(0), "segments");
  } else {
    TORCH_CHECK(seg_slot.size(0) <= proj.size(0), "rows");
  }
  const long ns = seg_slot.size(0);
  if (ns == 0) return;
  const bool vec = a.D % 4 == 0 && a.D <= 256 && a.stride % 4 == 0 &&
                   q_off % 4 == 0 && k_off % 4 == 0;
  by_dtype(proj, [&](auto t0) {
    using A = decltype(t0);
    auto run = [&](auto vec_, auto lpr_, auto epl_, auto ch_) {
      constexpr int LPR = decltype(lpr_)::value;
      const int rows = 1024 / LPR;
      linear_recurrent_kernel<A, decltype(vec_)::value, LPR,
                              decltype(epl_)::value, decltype(ch_)::value>
          <<<dim3(ns, a.H, (a.V + rows - 1) / rows), dim3(256), 0,
             current_stream()>>>(
              ptr<A>(o), ptr<A>(proj), a.stride, a.q_off, a.k_off, a.v_off,
              a.H, a.D, a.V, (int)act, (float)qscale, fptr(decay),
              fptr(state), seg_row0 ? iptr(*seg_row0) : nullptr,
              seg_row0 ? iptr(*seg_len) : nullptr, iptr(seg_slot),
              iptr(positions));
    };
    auto sized = [&](auto ch_) {
      using I1 = std::integral_constant<int, 1>;
      using I4 = std::integral_constant<int, 4>;
      using I8 = std::integral_constant<int, 8>;
      if (!vec) run(I1(), std::integral_constant<int, 64>(), I8(), ch_);
      else if (a.D <= 32) run(I4(), I8(), I1(), ch_);
      else if (a.D <= 64)
        run(I4(), std::integral_constant<int, 16>(), I1(), ch_);
      else if (a.D <= 128)
        run(I4(), std::integral_constant<int, 32>(), I1(), ch_);
      else run(I4(), std::integral_constant<int, 64>(), I1(), ch_);
    };
    if (channel) sized(std::true_type());
    else sized(std::false_type());
  });
  HIP_CHECK_KERNEL();
}

bool linear_tiles_ok(const Tensor &proj, const Tensor &state) {
  return proj.scalar_type() == torch::kBFloat16 && state.size(3) % 8 == 0 &&
         state.size(2) % 8 == 0 && state.size(3) <= 256 &&
         proj.size(1) % 8 == 0;
}

// decay: channel ? log decay summed along each chunk [rows, H*D]
//                : powers of each head's decay [H, LIN_CHUNK + 1]
void linear_chunked(Tensor o, Tensor proj, int64_t q_off, int64_t k_off,
                    int64_t v_off, int64_t act, double qscale, Tensor decay,
                    bool channel, Tensor state, Tensor chunk_row0,
                    Tensor chunk_len, Tensor seg_row0, Tensor seg_chunk0,
                    Tensor seg_slot, Tensor positions) {
  const LinDims a = lin_dims(o, proj, state, q_off, k_off, v_off);
  TORCH_CHECK(linear_tiles_ok(proj, state) && q_off % 8 == 0 &&
              k_off % 8 == 0 && v_off % 8 == 0,
              "linear_chunked: dtype, head sizes or offsets");
  check_decay(decay, a, proj.size(0), channel, LIN_CHUNK + 1);
  CHECK_I32(chunk_row0); CHECK_I32(chunk_len); CHECK_I32(seg_row0);
  CHECK_I32(seg_chunk0); CHECK_I32(seg_slot); CHECK_I32(positions);
  const long nc = chunk_row0.size(0), ns = seg_row0.size(0);
  TORCH_CHECK(chunk_len.size(0) == nc && seg_chunk0.size(0) == ns + 1 &&
              seg_slot.size(0) == ns, "chunk lists");
  if (nc == 0 || ns == 0) return;
  auto ws = torch::empty({nc, a.H, a.V, a.D},
                         proj.options().dtype(torch::kFloat32));
  auto stream = current_stream();
  const Tensor state_pool = state;
  const dim3 g_scan(ns, a.H, (a.V * a.D + 1023) / 1024);
  auto run = [&](auto ch_, auto nk_) {
    constexpr bool CH = decltype(ch_)::value;
    auto state = [&](auto td_, auto tv_) {
      constexpr int TD = decltype(td_)::value, TV = decltype(tv_)::value;
      const int tiles = ((a.D + TD - 1) / TD) * ((a.V + TV - 1) / TV);
      linear_chunk_state_kernel<CH, TD, TV>
          <<<dim3(nc, a.H, tiles), dim3(256), 0, stream>>>(
              fptr(ws), ptr<bf16>(proj), a.stride, a.k_off, a.v_off, a.H,
              a.D, a.V, (int)act, fptr(decay), iptr(chunk_row0),
              iptr(chunk_len));
    };
    if (a.V <= 64) state(Int<64>(), Int<64>());
    else state(Int<64>(), Int<128>());
    HIP_CHECK_KERNEL();
    linear_chunk_scan_kernel<CH><<<g_scan, dim3(256), 0, stream>>>(
        fptr(ws), fptr(state_pool), a.H, a.D, a.V, fptr(decay), iptr(chunk_row0),
        iptr(chunk_len), iptr(seg_row0), iptr(seg_chunk0), iptr(seg_slot),
        iptr(positions));
    HIP_CHECK_KERNEL();
    linear_chunk_out_kernel<CH, decltype(nk_)::value>
        <<<dim3(nc, a.H), dim3(256), 0, stream>>>(
            ptr<bf16>(o), fptr(ws), ptr<bf16>(proj), a.stride, a.q_off,
            a.k_off, a.v_off, a.H, a.D, a.V, (int)act, (float)qscale,
            fptr(decay), iptr(chunk_row0), iptr(chunk_len));
    HIP_CHECK_KERNEL();
  };
  auto sized = [&](auto ch_) {
    if (a.D <= 32) run(ch_, std::integral_constant<int, 1>());
    else if (a.D <= 64) run(ch_, std::integral_constant<int, 2>());
    else if (a.D <= 128) run(ch_, std::integral_constant<int, 4>());
    else run(ch_, std::integral_constant<int, 8>());
  };
  if (channel) sized(std::true_type());
  else sized(std::false_type());
}

#include "hybrid_forward.h"
#include "hybrid_blocks.h"

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.attr("LIN_CHUNK") = LIN_CHUNK;
  m.def("post_norm", &post_norm, "Residual sum and RMS norm after it");
  m.def("glu", &glu, "SiLU(gate) * up");
  m.def("gated_norm", &gated_norm, "Grouped RMS norm times a gate");
  m.def("qk_norm_rope_store", &qk_norm_rope_store,
        "Whole-projection QK norm, interleaved RoPE, paged store (V = raw K)");
  m.def("log_decay", &log_decay, "Low-rank sigmoid decay, log, run sums");
  m.def("local_attn_rows", &local_attn_rows,
        "Chunk-local sink attention, any head dim, bf16/float32");
  m.def("local_attn_prefill", &local_attn_prefill,
        "Chunk-local sink attention, matrix-core prefill tiles");
  m.def("local_attn_decode", &local_attn_decode,
        "Chunk-local sink attention, matrix-core flash-decode");
  m.def("attn_tiles_ok", &attn_tiles_ok, "Matrix-core attention applies");
  m.def("linear_recurrent", &linear_recurrent,
        "Linear attention token by token (decode, float32)");
  m.def("linear_chunked", &linear_chunked,
        "Chunked linear attention on the matrix cores (bf16 prefill)");
  m.def("linear_tiles_ok", &linear_tiles_ok, "Chunked form applies");
  qhybrid::bind(m);
}
