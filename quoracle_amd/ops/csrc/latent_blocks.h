// Blocks of models with norms before and after each sublayer: latent attention
// ("lat.*"), a gelu feed-forward ("mlp.*") and a mixture of experts ("moe.*").
// Each adds its normed output to the stream and leaves the input of the block
// behind it.
//
// Included by latent_bindings.cpp after the kernel wrappers it calls.
#pragma once

namespace qhybrid {

struct SandwichBlock : Block {
  Tensor post;                  // norm of the output
  void add(const Model &m, Stream &s, const Next &next, const Tensor &y,
           const Tensor &bias, const Tensor &y2, const Tensor &gate) const {
    sandwich_norm(s.x, s.h, next.join ? OptTensor(s.joined) : c10::nullopt,
                  opt(next.norm), y, opt(bias), opt(y2), opt(gate), post,
                  m.eps);
  }
};

struct LatentBlock : SandwichBlock {
  int64_t H, dim, vdim, rank, kv_off;
  double scale;
  Tensor w_in, w_uq, w_kv, w_uk_t, w_o, q_norm, kv_norm, freq, sink;

  LatentBlock(const Tensors &t, const Numbers &n)
      : H(n.at("lat.heads")), dim(n.at("lat.dim")), vdim(n.at("lat.vdim")),
        rank(n.at("lat.rank")), kv_off(n.at("lat.kv_off")),
        scale(n.at("lat.scale")), w_in(t.at("lat.w_in")),
        w_uq(t.at("lat.w_uq")), w_kv(t.at("lat.w_kv")),
        w_uk_t(t.at("lat.w_uk_t")), w_o(t.at("lat.w_o")),
        q_norm(t.at("lat.q_norm")), kv_norm(t.at("lat.kv_norm")),
        freq(t.at("lat.freq")), sink(find_or_none(t, "lat.sink")) {}

  void run(const Model &m, const Run &r, const Batch &b, const Pools &pools,
           Stream &s, const Next &next) const override {
    const Tensor &pool = pools.at("latent").at(r.latent);
    auto proj = at::linear(s.h, w_in);
    auto cq = torch::empty({b.rows, q_norm.size(0)}, proj.options());
    latent_store(cq, pool, proj, kv_off, rank, q_norm, kv_norm,
                 b.at("positions"), b.at("slots"), freq, m.eps);
    auto q = at::linear(cq, w_uq).view({b.rows, H, -1});
    rotate_heads(q, dim, b.at("positions"), freq);
    auto out = torch::empty({b.rows, H, vdim}, proj.options());
    latent_attend(out, q, pool, w_kv, w_uk_t, opt(sink), scale, b);
    add(m, s, next, at::linear(out.view({b.rows, H * vdim}), w_o), {}, {}, {});
  }
};

inline Tensor gelu_mlp(const Tensor &h, const Tensor &up, const Tensor &up_b,
                       const Tensor &down) {
  auto z = at::linear(h, up);
  bias_gelu(z, opt(up_b));
  return at::linear(z, down);
}

struct MlpBlock : SandwichBlock {
  Tensor up, up_b, down, down_b;

  void run(const Model &m, const Run &, const Batch &, const Pools &,
           Stream &s, const Next &next) const override {
    add(m, s, next, gelu_mlp(s.h, up, up_b, down), down_b, {}, {});
  }
};

struct MoeBlock : SandwichBlock {
  int64_t top;
  Tensor router, up, down, shared_up, shared_down;

  void run(const Model &m, const Run &, const Batch &b, const Pools &,
           Stream &s, const Next &next) const override {
    auto f32 = s.x.options();
    auto ids = torch::empty({b.rows, top}, f32.dtype(torch::kInt32));
    auto weights = torch::empty({b.rows, top}, f32);
    Tensor gate, shared;
    if (shared_up.defined()) gate = torch::empty({b.rows}, f32);
    moe_route(ids, weights, opt(gate), s.h, router, up.size(0));
    if (shared_up.defined())
      shared = gelu_mlp(s.h, shared_up, Tensor(), shared_down);
    auto y = torch::empty({b.rows, top, s.h.size(1)}, s.h.options());
    moe_experts(y, s.h, ids, weights, up, down);
    add(m, s, next, y, {}, shared, gate);
  }
};

Layer make_layer(const Tensors &t, const Numbers &n) {
  Layer blocks;
  if (!t.count("lat.w_in")) return blocks;
  auto mixer = std::make_shared<LatentBlock>(t, n);
  mixer->pre = t.at("norm1");
  mixer->post = t.at("norm1b");
  blocks.push_back(mixer);
  if (t.count("mlp.up")) {
    auto ff = std::make_shared<MlpBlock>();
    ff->up = t.at("mlp.up");
    ff->down = t.at("mlp.down");
    ff->up_b = find_or_none(t, "mlp.up_b");
    ff->down_b = find_or_none(t, "mlp.down_b");
    ff->pre = t.at("norm2");
    ff->post = t.at("norm2b");
    blocks.push_back(ff);
  } else if (t.count("moe.up")) {
    auto ff = std::make_shared<MoeBlock>();
    ff->top = n.at("moe.top");
    ff->router = t.at("moe.router");
    ff->up = t.at("moe.up");
    ff->down = t.at("moe.down");
    ff->shared_up = find_or_none(t, "moe.shared_up");
    ff->shared_down = find_or_none(t, "moe.shared_down");
    ff->pre = t.at("norm2");
    ff->post = t.at("norm2b");
    blocks.push_back(ff);
  }
  return blocks;
}

}  // namespace qhybrid
