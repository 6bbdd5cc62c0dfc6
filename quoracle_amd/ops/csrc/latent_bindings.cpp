// Torch bindings of latent attention, of mixtures of experts, and of the norms
// around them, for bf16 and float32 activations (gfx950).  One translation
// unit, built in-tree by quoracle_amd/ops/build.py.

#include <torch/extension.h>

#include <c10/hip/HIPStream.h>

#include <stdexcept>
#include <string>

#include "stream_kernels.hip"
#include "latent_elementwise.hip"
#include "latent_attention.hip"
#include "moe.hip"

namespace {

#include "hybrid_host.h"

void sandwich_norm(Tensor x, Tensor h, OptTensor joined, OptTensor w_next,
                   Tensor y, OptTensor bias, OptTensor y2, OptTensor gate,
                   Tensor w, double eps) {
  CHECK_F32(x); CHECK_GPU(h); CHECK_GPU(y); CHECK_F32(w);
  const int n = w.size(0);
  const long T = x.numel() / n;
  const long K = y.dim() == 3 ? y.size(1) : 1;
  TORCH_CHECK(x.numel() == T * n && h.numel() == T * n &&
              y.numel() == T * K * n, "sandwich_norm shapes");
  if (joined) {
    CHECK_GPU(*joined);
    TORCH_CHECK(joined->numel() == 2 * T * n, "sandwich_norm joined");
  }
  if (w_next) { CHECK_F32(*w_next); TORCH_CHECK(w_next->numel() == n, "next"); }
  if (bias) { CHECK_F32(*bias); TORCH_CHECK(bias->numel() == n, "bias"); }
  TORCH_CHECK(y2.has_value() == gate.has_value(), "y2 and gate");
  if (y2) {
    CHECK_GPU(*y2); CHECK_F32(*gate);
    TORCH_CHECK(y2->numel() == T * n && gate->numel() == T, "sandwich_norm y2");
  }
  if (T == 0) return;
  by_dtype(h, [&](auto t0) {
    using A = decltype(t0);
    by_vec(n % 8 == 0, [&](auto v) {
      by_items(n, v, [&](auto ni) {
        sandwich_norm_kernel<A, decltype(v)::value, decltype(ni)::value>
            <<<dim3(T), dim3(256), 0, current_stream()>>>(
                fptr(x), ptr<A>(h), joined ? ptr<A>(*joined) : nullptr,
                w_next ? fptr(*w_next) : nullptr, ptr<A>(y), (int)K,
                bias ? fptr(*bias) : nullptr, y2 ? ptr<A>(*y2) : nullptr,
                gate ? fptr(*gate) : nullptr, fptr(w), n, (float)eps);
      });
    });
  });
  HIP_CHECK_KERNEL();
}

const double *freq_ptr(const Tensor &freq) {
  CHECK_GPU(freq);
  TORCH_CHECK(freq.scalar_type() == torch::kFloat64 && freq.numel() <= 2048,
              "freq must be float64");
  return freq.data_ptr<double>();
}

void latent_store(Tensor cq, Tensor pool, Tensor proj, int64_t kv_off,
                  int64_t rank_p, Tensor wq, Tensor wkv, Tensor positions,
                  Tensor slots, Tensor freq, double eps) {
  CHECK_GPU(cq); CHECK_GPU(pool); CHECK_GPU(proj); CHECK_F32(wq);
  CHECK_F32(wkv); CHECK_I32(positions); CHECK_I32(slots);
  const long T = proj.size(0), stride = proj.size(1);
  const int q_rank = wq.size(0), rank = wkv.size(0), pairs = freq.size(0);
  const int width = pool.size(2);
  TORCH_CHECK(pool.dim() == 3 && rank <= rank_p &&
              rank_p + 2 * pairs <= width, "latent_store pool");
  TORCH_CHECK(cq.numel() == T * q_rank && q_rank <= kv_off &&
              kv_off + rank + 2 * pairs <= stride &&
              positions.size(0) == T && slots.size(0) == T,
              "latent_store shapes");
  const double *f = freq_ptr(freq);
  if (T == 0) return;
  const bool vec = q_rank % 8 == 0 && rank % 8 == 0 && kv_off % 8 == 0 &&
                   stride % 8 == 0 && width % 8 == 0;
  by_dtype(proj, [&](auto t0) {
    using A = decltype(t0);
    by_vec(vec, [&](auto v) {
      latent_store_kernel<A, decltype(v)::value>
          <<<dim3(T), dim3(256), 2 * pairs * sizeof(float),
             current_stream()>>>(
              ptr<A>(cq), ptr<A>(pool), ptr<A>(proj), stride, q_rank,
              (int)kv_off, rank, (int)rank_p, width, fptr(wq), fptr(wkv),
              iptr(positions), iptr(slots), f, pairs, (float)eps);
    });
  });
  HIP_CHECK_KERNEL();
}

void rotate_heads(Tensor q, int64_t off, Tensor positions, Tensor freq) {
  CHECK_GPU(q); CHECK_I32(positions);
  const long T = q.size(0);
  const int H = q.size(1), D = q.size(2), pairs = freq.size(0);
  TORCH_CHECK(off + 2 * pairs <= D && positions.size(0) == T,
              "rotate_heads shapes");
  const double *f = freq_ptr(freq);
  if (T == 0 || pairs == 0) return;
  by_dtype(q, [&](auto t0) {
    using A = decltype(t0);
    auto run = [&](auto kernel) {
      kernel<<<dim3(T), dim3(256), 2 * pairs * sizeof(float),
               current_stream()>>>(ptr<A>(q), H, D, (int)off,
                                   iptr(positions), f, pairs);
    };
    if (pairs % 4 == 0 && D % 8 == 0 && off % 8 == 0)
      run(rotate_heads_kernel<A, 4>);
    else run(rotate_heads_kernel<A, 1>);
  });
  HIP_CHECK_KERNEL();
}

void bias_gelu(Tensor z, OptTensor bias) {
  CHECK_GPU(z);
  const int n = z.size(-1);
  const long T = z.numel() / n;
  if (bias) { CHECK_F32(*bias); TORCH_CHECK(bias->numel() == n, "bias_gelu"); }
  if (T == 0) return;
  by_dtype(z, [&](auto t0) {
    using A = decltype(t0);
    by_vec(n % 8 == 0, [&](auto v) {
      constexpr int VEC = decltype(v)::value;
      bias_gelu_kernel<A, VEC>
          <<<dim3(T, (n + 256 * VEC - 1) / (256 * VEC)), dim3(256), 0,
             current_stream()>>>(ptr<A>(z), bias ? fptr(*bias) : nullptr, n);
    });
  });
  HIP_CHECK_KERNEL();
}

// -- grouped products --------------------------------------------------------

bool gg_vectors_ok(const GroupedGemm &p) {
  return p.K % 8 == 0 && p.lda % 8 == 0 && p.a_group % 8 == 0;
}

// Rows per tile that suit `rows` rows per group on average.
int gg_tile_rows(bool vec, long rows) {
  return !vec || rows <= 32 ? 16 : rows <= 96 ? 64 : rows < 1024 ? 128 : 256;
}

// `tiles` row tiles of BM rows (of every group, if there is no tile list).
template <typename A>
void gg_launch(GroupedGemm p, int BM, long tiles, long groups, bool vec) {
  if (tiles == 0 || groups == 0 || p.N == 0) return;
  TORCH_CHECK(tiles <= 65535 && groups <= 65535, "grouped product grid");
  p.row_tiles = tiles;
  auto run = [&](auto kernel, int cols) {
    kernel<<<dim3((p.N + cols - 1) / cols, tiles, groups), dim3(256), 0,
             current_stream()>>>(p);
    HIP_CHECK_KERNEL();
  };
  auto run_tiles = [&](auto kernel, int cols, int threads) {
    const long all = (p.N + cols - 1) / cols * tiles;
    TORCH_CHECK(all < 1L << 31, "grouped product grid");
    kernel<<<dim3(all, 1, groups), dim3(threads), 0, current_stream()>>>(p);
    HIP_CHECK_KERNEL();
  };
  if constexpr (sizeof(A) == 2) {
    if (vec) {
      if (BM == 256) run_tiles(gg_tile_kernel<256, 256, 2, 4>, 256, 512);
      else if (BM == 128) run_tiles(gg_tile_kernel<128, 128, 2, 2>, 128, 256);
      else if (BM == 64) run_tiles(gg_tile_kernel<64, 128, 2, 2>, 128, 256);
      else if (p.K > 256) run(gg_strip_kernel<true>, 32);
      else run(gg_strip_kernel<false>, 128);
      return;
    }
  }
  TORCH_CHECK(BM == 16, "grouped product tile");
  run(gg_plain_kernel<A>, 64);
}

// c[t, h, :] = w[h] a[t, h, :a_off + K] for the first `rows` tokens, from
// column a_off of every head of a.
void head_product(const Tensor &c, const Tensor &a, int64_t a_off,
                  const Tensor &w, int64_t rows) {
  CHECK_GPU(c); CHECK_GPU(a); CHECK_GPU(w);
  const int H = w.size(0), N = w.size(1), K = w.size(2);
  TORCH_CHECK(a.size(1) == H && c.size(1) == H && c.size(2) == N &&
              a_off + K <= a.size(2) && a.size(0) >= rows &&
              c.size(0) >= rows, "head_product shapes");
  if (rows == 0) return;
  by_dtype(a, [&](auto t0) {
    using A = decltype(t0);
    GroupedGemm p{};
    p.a = ptr<A>(a) + a_off;
    p.b = ptr<A>(w);
    p.c = ptr<A>(c);
    p.lda = H * a.size(2);
    p.a_group = a.size(2);
    p.ldc = (long)H * N;
    p.c_group = N;
    p.M = rows;
    p.N = N;
    p.K = K;
    const bool vec = gg_vectors_ok(p) && a_off % 8 == 0;
    // few columns: short tiles, so that there are enough of them
    const int BM = rows <= 64 ? 16 : gg_tile_rows(vec && sizeof(A) == 2, rows);
    gg_launch<A>(p, BM, (rows + BM - 1) / BM, H, vec);
  });
}

// -- latent attention --------------------------------------------------------

struct LatentDims {
  int H, QP, dim, rot, rank, vdim, BS, MAXB;
};

// Workgroups that fill the chip, two on a CU.
constexpr long LATENT_GROUPS = 512;

// Rows of one launch in the latent space: decode rows (tiles undefined), or
// tiles of at most 16 tokens.
void latent_tiles(const Tensor &o, const Tensor &q_lat, const Tensor &q,
                  const Tensor &pool, const OptTensor &sink, double scale,
                  const LatentDims &d, const Tensor &bt, const Tensor &ctx,
                  const Tensor *tiles, long n_tiles, int tokens, long seen) {
  if (n_tiles == 0) return;
  const long rows = (long)tokens * d.H;        // flattened rows of a tile
  const int MT = rows <= 32 ? 2 : 4;
  const long parts = (rows + 16 * MT - 1) / (16 * MT);
  const long ns = std::max<long>(
      1, std::min<long>({LATENT_GROUPS * 2 / MT / (n_tiles * parts), seen / 64,
                         64}));
  Tensor pm, pl, pa;
  if (ns > 1) {
    auto opts = q.options().dtype(torch::kFloat32);
    pm = torch::empty({o.size(0), d.H, ns}, opts);
    pl = torch::empty({o.size(0), d.H, ns}, opts);
    pa = torch::empty({o.size(0), d.H, ns, d.rank}, opts);
  }
  auto run = [&](auto rp, auto mt) {
    constexpr int RP = decltype(rp)::value, M = decltype(mt)::value;
    latent_tile_kernel<RP, M>
        <<<dim3(n_tiles, parts, ns), dim3(64 * latent_waves<M>()), 0,
           current_stream()>>>(
            ptr<bf16>(o), ns > 1 ? fptr(pm) : nullptr,
            ns > 1 ? fptr(pl) : nullptr, ns > 1 ? fptr(pa) : nullptr,
            ptr<bf16>(q_lat), ptr<bf16>(q), ptr<bf16>(pool), iptr(bt),
            tiles ? nullptr : iptr(ctx), tiles ? iptr(tiles[0]) : nullptr,
            tiles ? iptr(tiles[1]) : nullptr, tiles ? iptr(tiles[2]) : nullptr,
            tiles ? iptr(tiles[3]) : nullptr, sink ? fptr(*sink) : nullptr,
            (float)scale, d.H, d.rank, d.rot, d.QP, d.dim,
            __builtin_ctz(d.BS), d.MAXB, (int)ns);
  };
  auto sized = [&](auto rp) {
    if (MT == 2) run(rp, Int<2>());
    else run(rp, Int<4>());
  };
  if (d.rank <= 64) sized(Int<64>());
  else if (d.rank <= 128) sized(Int<128>());
  else if (d.rank <= 256) sized(Int<256>());
  else sized(Int<512>());
  HIP_CHECK_KERNEL();
  if (ns == 1) return;
  // decode rows come first, portions behind them
  const long first = tiles ? ctx.size(0) : 0;
  const long n = tiles ? o.size(0) - first : ctx.size(0);
  const long at = first * d.H;
  latent_combine_kernel<<<dim3(n, d.H, (d.rank + 127) / 128), dim3(128),
                          ns * sizeof(float), current_stream()>>>(
      ptr<bf16>(o) + at * d.rank, fptr(pm) + at * ns, fptr(pl) + at * ns,
      fptr(pa) + at * ns * d.rank, d.H, d.rank, (int)ns);
  HIP_CHECK_KERNEL();
}

// Long portions: rows of q behind the latent-space ones, in 128-row tiles.
void expanded_prefill(const Tensor &out, const Tensor &q, const Tensor &pool,
                      const Tensor &w_kv, const OptTensor &sink, double scale,
                      const LatentDims &d, const Tensor &slots,
                      const Tensor &q0, const Tensor &qn, const Tensor &pos0,
                      const Tensor &ctx0, long max_kv) {
  CHECK_I32(slots); CHECK_I32(q0); CHECK_I32(qn); CHECK_I32(pos0);
  CHECK_I32(ctx0);
  TORCH_CHECK(d.QP <= 256 && d.vdim <= 256, "expanded_prefill head sizes");
  const long n = slots.size(0), nt = q0.size(0);
  TORCH_CHECK(qn.size(0) == nt && pos0.size(0) == nt && ctx0.size(0) == nt,
              "expanded_prefill tiles");
  if (nt == 0) return;
  const int width = d.rank + d.rot;
  auto ctx = torch::empty({n, width}, pool.options());
  gather_latents_kernel<<<dim3(n), dim3(64), 0, current_stream()>>>(
      ptr<bf16>(ctx), ptr<bf16>(pool), iptr(slots), width);
  HIP_CHECK_KERNEL();
  auto kv = at::linear(ctx.narrow(1, 0, d.rank), w_kv);
  const long ns = max_kv < 1024 ? 1 : std::max<long>(
      1, std::min<long>({LATENT_GROUPS / (nt * d.H), max_kv / 256, 16}));
  Tensor pm, pl, pa;
  if (ns > 1) {
    auto opts = q.options().dtype(torch::kFloat32);
    pm = torch::empty({nt, d.H, ns, 128}, opts);
    pl = torch::empty({nt, d.H, ns, 128}, opts);
    pa = torch::empty({nt, d.H, ns, 128, d.vdim}, opts);
  }
  auto run = [&](auto dq, auto dv) {
    expanded_prefill_kernel<decltype(dq)::value, decltype(dv)::value>
        <<<dim3(nt * d.H, ns), dim3(256), 0, current_stream()>>>(
            ptr<bf16>(out), ns > 1 ? fptr(pm) : nullptr,
            ns > 1 ? fptr(pl) : nullptr, ns > 1 ? fptr(pa) : nullptr,
            ptr<bf16>(q), ptr<bf16>(ctx), ptr<bf16>(kv), iptr(q0), iptr(qn),
            iptr(pos0), iptr(ctx0), sink ? fptr(*sink) : nullptr,
            (float)scale, (int)nt, d.H, d.dim, d.rot, d.vdim, d.rank,
            (int)ns);
  };
  if (d.QP <= 64 && d.vdim <= 64) run(Int<64>(), Int<64>());
  else if (d.QP <= 128 && d.vdim <= 128) run(Int<128>(), Int<128>());
  else if (d.QP <= 192 && d.vdim <= 128) run(Int<192>(), Int<128>());
  else run(Int<256>(), Int<256>());
  HIP_CHECK_KERNEL();
  if (ns == 1) return;
  expanded_combine_kernel<<<dim3(nt, d.H, 128), dim3(64), 0,
                            current_stream()>>>(
      ptr<bf16>(out), fptr(pm), fptr(pl), fptr(pa), iptr(q0), iptr(qn), d.H,
      d.vdim, (int)ns);
  HIP_CHECK_KERNEL();
}

#include "hybrid_forward.h"

// Attention of every row of a batch over the paged latents: decode rows and
// short portions in the latent space, long portions over expanded keys and
// values; everything in the latent space on the vector ALU where the matrix
// kernels do not apply.
void latent_attend(const Tensor &out, const Tensor &q, const Tensor &pool,
                   const Tensor &w_kv, const Tensor &w_uk_t,
                   const OptTensor &sink, double scale,
                   const qhybrid::Batch &b) {
  CHECK_GPU(out); CHECK_GPU(q); CHECK_GPU(pool); CHECK_GPU(w_kv);
  CHECK_GPU(w_uk_t);
  const Tensor &bt = b.at("block_tables");
  CHECK_I32(bt);
  LatentDims d{};
  d.H = q.size(1);
  d.QP = q.size(2);
  d.rank = w_uk_t.size(1);
  d.dim = w_uk_t.size(2);
  d.vdim = out.size(2);
  d.rot = pool.size(2) - d.rank;
  d.BS = pool.size(1);
  d.MAXB = bt.size(1);
  const long T = q.size(0);
  TORCH_CHECK(w_uk_t.size(0) == d.H && d.dim + d.rot == d.QP &&
              w_kv.size(0) == (long)d.H * (d.dim + d.vdim) &&
              w_kv.size(1) == d.rank && out.size(0) == T &&
              out.size(1) == d.H && T == b.rows,
              "latent attention shapes");
  TORCH_CHECK(d.rank % 8 == 0 && d.rot % 8 == 0 && d.dim % 8 == 0 &&
              d.vdim % 8 == 0, "latent attention sizes are padded to 8");
  if (sink) { CHECK_F32(*sink); TORCH_CHECK(sink->numel() == d.H, "sink"); }
  // a batch with portions that names neither short tiles nor contexts is one
  // of a model with other layers that the matrix kernels do not take
  const bool tiles = q.scalar_type() == torch::kBFloat16 && d.rank <= 512 &&
                     d.rot <= 64 && (d.BS & (d.BS - 1)) == 0 &&
                     (T == b.n_decode || b.n_latent > b.n_decode ||
                      b.has("ctx_slots"));
  const long n = tiles ? b.n_latent : T;
  TORCH_CHECK(b.n_decode <= n && n <= T, "latent attention rows");
  auto w_uv = w_kv.narrow(0, (long)d.H * d.dim, (long)d.H * d.vdim)
                  .view({d.H, d.vdim, d.rank});
  if (n > 0) {
    auto q_lat = torch::empty({n, d.H, d.rank}, q.options());
    auto o = torch::empty({n, d.H, d.rank}, q.options());
    head_product(q_lat, q, 0, w_uk_t, n);
    if (tiles) {
      Tensor ctx = b.n_decode ? b.at("ctx_lens") : bt.new_empty({0});
      CHECK_I32(ctx);
      TORCH_CHECK(ctx.size(0) == b.n_decode, "ctx_lens");
      latent_tiles(o, q_lat, q, pool, sink, scale, d, bt, ctx, nullptr,
                   b.n_decode, 1, b.max_ctx);
      if (n > b.n_decode) {
        const Tensor t[4] = {b.at("short_q0"), b.at("short_qn"),
                             b.at("short_seq"), b.at("short_pos0")};
        for (const Tensor &x : t) { CHECK_I32(x); }
        latent_tiles(o, q_lat, q, pool, sink, scale, d, bt, ctx, t,
                     t[0].size(0), 16, b.max_kv);
      }
    } else {
      const Tensor &seq = b.at("row_seq"), &pos = b.at("positions");
      CHECK_I32(seq); CHECK_I32(pos);
      const size_t lds = (2 * d.rank + d.rot) * sizeof(float);
      TORCH_CHECK(lds <= 60000, "latent of more than 7000 values");
      by_dtype(q, [&](auto t0) {
        using A = decltype(t0);
        latent_rows_kernel<A>
            <<<dim3(T, d.H), dim3(128), lds, current_stream()>>>(
                ptr<A>(o), ptr<A>(q_lat), ptr<A>(q), ptr<A>(pool), iptr(bt),
                iptr(seq), iptr(pos), sink ? fptr(*sink) : nullptr,
                (float)scale, d.H, d.rank, d.rot, d.QP, d.dim, d.BS, d.MAXB);
      });
      HIP_CHECK_KERNEL();
    }
    head_product(out, o, 0, w_uv, n);
  }
  if (n < T)
    expanded_prefill(out, q, pool, w_kv, sink, scale, d, b.at("ctx_slots"),
                     b.at("tile_q0"), b.at("tile_qn"), b.at("tile_pos0"),
                     b.at("tile_ctx0"), b.max_kv);
}

void latent_attention(Tensor out, Tensor q, Tensor pool, Tensor w_kv,
                      Tensor w_uk_t, OptTensor sink, double scale,
                      const qhybrid::Tensors &tensors,
                      const qhybrid::Counts &counts) {
  latent_attend(out, q, pool, w_kv, w_uk_t, sink, scale,
                qhybrid::make_batch(tensors, counts, q.size(0)));
}

// -- mixture of experts ------------------------------------------------------

void moe_route(Tensor ids, Tensor weights, OptTensor gate, Tensor h,
               Tensor router, int64_t experts) {
  CHECK_I32(ids); CHECK_F32(weights); CHECK_GPU(h); CHECK_GPU(router);
  const long T = h.size(0);
  const int n = h.size(1), E = experts, top = ids.size(1);
  TORCH_CHECK(ids.numel() == T * top && weights.numel() == T * top &&
              router.size(1) == n && top >= 1 && top <= E &&
              router.size(0) >= E + (gate ? 1 : 0), "moe_route shapes");
  if (gate) { CHECK_F32(*gate); TORCH_CHECK(gate->numel() == T, "gate"); }
  TORCH_CHECK(E <= 1024, "more than 1024 experts");
  if (T == 0) return;
  float *g = gate ? fptr(*gate) : nullptr;
  if (h.scalar_type() == torch::kBFloat16 && n % 8 == 0 && E <= 384) {
    moe_route_mfma_kernel<<<dim3((T + 15) / 16), dim3(512),
                            16 * (E + 1) * sizeof(float), current_stream()>>>(
        ids.data_ptr<int>(), fptr(weights), g, ptr<bf16>(h),
        ptr<bf16>(router), (int)T, n, E, top);
  } else {
    by_dtype(h, [&](auto t0) {
      using A = decltype(t0);
      by_vec(n % 8 == 0, [&](auto v) {
        moe_route_kernel<A, decltype(v)::value>
            <<<dim3(T), dim3(256), E * sizeof(float), current_stream()>>>(
                ids.data_ptr<int>(), fptr(weights), g, ptr<A>(h),
                ptr<A>(router), n, E, top);
      });
    });
  }
  HIP_CHECK_KERNEL();
}

void moe_experts(Tensor y, Tensor h, Tensor ids, Tensor weights, Tensor up,
                 Tensor down) {
  CHECK_GPU(y); CHECK_GPU(h); CHECK_I32(ids); CHECK_F32(weights);
  CHECK_GPU(up); CHECK_GPU(down);
  const long T = h.size(0), top = ids.size(1), S = T * top;
  const int n = h.size(1), E = up.size(0), ff = up.size(1);
  TORCH_CHECK(up.size(2) == n && down.size(0) == E && down.size(1) == n &&
              down.size(2) == ff && y.numel() == S * n &&
              ids.numel() == S && weights.numel() == S && E <= 4096,
              "moe_experts shapes");
  if (S == 0) return;
  by_dtype(h, [&](auto t0) {
    using A = decltype(t0);
    const bool vec = sizeof(A) == 2 && n % 8 == 0 && ff % 8 == 0;
    const int BM = gg_tile_rows(vec, (S + E - 1) / E);
    const long nt = S / BM + std::min<long>(E, S);
    auto list = torch::empty({S + 3 * nt + 1}, ids.options());
    int *rows = list.data_ptr<int>();
    int *tg = rows + S, *tr0 = tg + nt, *trn = tr0 + nt, *count = trn + nt;
    moe_order_kernel<<<dim3(1), dim3(1024), 3 * E * sizeof(int),
                       current_stream()>>>(rows, tg, tr0, trn, count,
                                           iptr(ids), (int)S, E, BM, (int)nt);
    HIP_CHECK_KERNEL();
    auto act = torch::empty({S, ff}, h.options());
    GroupedGemm p{};
    p.a = ptr<A>(h);
    p.b = ptr<A>(up);
    p.c = ptr<A>(act);
    p.lda = n;
    p.ldc = ff;
    p.N = ff;
    p.K = n;
    p.tile_group = tg;
    p.tile_row0 = tr0;
    p.tile_rows = trn;
    p.tile_count = count;
    p.rows = rows;
    p.a_div = top;
    p.scale = fptr(weights);
    p.gelu = true;
    gg_launch<A>(p, BM, nt, 1, vec);
    p.a = ptr<A>(act);
    p.b = ptr<A>(down);
    p.c = ptr<A>(y);
    p.lda = ff;
    p.ldc = n;
    p.N = n;
    p.K = ff;
    p.a_div = 0;
    p.c_slot = true;
    p.scale = nullptr;
    p.gelu = false;
    gg_launch<A>(p, BM, nt, 1, vec);
  });
}

#include "latent_blocks.h"

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("sandwich_norm", &sandwich_norm,
        "Residual sum of a normed sublayer output, and the next norm");
  m.def("latent_store", &latent_store,
        "Norm of both latents, rotated key part, paged store");
  m.def("rotate_heads", &rotate_heads, "Interleaved rotation in place");
  m.def("bias_gelu", &bias_gelu, "Exact gelu of z + bias in place");
  m.def("latent_attention", &latent_attention,
        "Sink attention of a mixed batch over paged latents");
  m.def("moe_route", &moe_route, "Sigmoid scores and the largest of them");
  m.def("moe_experts", &moe_experts,
        "Grouped products of the chosen experts, weights on their inputs");
  qhybrid::bind(m);
}
