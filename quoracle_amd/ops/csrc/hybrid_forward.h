// Native layer loop of the hybrid models (recurrent mixers, chunk-local
// attention, gated feed-forward, norm after the sum).
//
// A layer is described by a map of tensors and a map of numbers.  A mixer may
// hold a chunk-local attention part ("attn.*") and a linear-attention part
// ("lin.*"), both reading the rows of one fused input projection `w_in`; each
// has its own output projection, and the norm kernel joins them with their
// scales.  Plain matrix products go to the vendor library.
//
// Included by hybrid_bindings.cpp after the kernel wrappers it calls.
#pragma once

#include <map>
#include <unordered_map>
#include <vector>

namespace qhybrid {

using Tensors = std::map<std::string, Tensor>;
using Numbers = std::map<std::string, double>;

struct Attn {
  int64_t q_off, k_off, H, D, chunk, cache;
  double scale, mag, out_scale;
  bool sink;
  Tensor q_norm, k_norm, freq, w_o;
};

struct Linear {
  int64_t q_off, k_off, v_off, g_off, a_off, H, V, act, gate_act, groups,
      state;
  double qscale, tau, out_scale;
  bool channel;                 // decay per key channel and token
  Tensor w_o, norm;
  Tensor decay, powers;         // one constant per head
  Tensor a2, a2_b;              // channel: low-rank decay
};

struct Layer {
  Tensor w_in, norm1;
  bool has_attn, has_lin, has_mlp;
  Attn attn;
  Linear lin;
  Tensor gate_up, down, norm2;
};

struct Model {
  Tensor embed, pos, head, final_norm;
  double alpha, eps;
  std::vector<Layer> layers;
};

inline std::unordered_map<std::string, Model> &registry() {
  static std::unordered_map<std::string, Model> models;
  return models;
}

inline void register_model(const std::string &key, const Tensors &t,
                           const Numbers &n,
                           const std::vector<Tensors> &layer_tensors,
                           const std::vector<Numbers> &layer_numbers) {
  Model m;
  m.embed = t.at("embed");
  if (t.count("pos")) m.pos = t.at("pos");
  m.head = t.at("head");
  m.final_norm = t.at("final_norm");
  m.alpha = n.at("alpha");
  m.eps = n.at("eps");
  TORCH_CHECK(layer_tensors.size() == layer_numbers.size(), "layers");
  for (size_t i = 0; i < layer_tensors.size(); ++i) {
    const Tensors &lt = layer_tensors[i];
    const Numbers &ln = layer_numbers[i];
    auto num = [&](const char *k) { return ln.at(k); };
    auto ten = [&](const char *k) {
      auto it = lt.find(k);
      return it == lt.end() ? Tensor() : it->second;
    };
    Layer L;
    L.w_in = lt.at("w_in");
    L.norm1 = lt.at("norm1");
    L.has_attn = lt.count("attn.w_o");
    L.has_lin = lt.count("lin.w_o");
    L.has_mlp = lt.count("gate_up");
    TORCH_CHECK(L.has_attn || L.has_lin, "layer without a mixer");
    if (L.has_attn) {
      Attn &a = L.attn;
      a.q_off = num("attn.q_off");
      a.k_off = num("attn.k_off");
      a.H = num("attn.heads");
      a.D = num("attn.dim");
      a.chunk = num("attn.chunk");
      a.cache = num("attn.cache");
      a.scale = num("attn.scale");
      a.mag = num("attn.mag");
      a.out_scale = num("attn.out_scale");
      a.sink = num("attn.sink") != 0;
      a.q_norm = lt.at("attn.q_norm");
      a.k_norm = lt.at("attn.k_norm");
      a.freq = lt.at("attn.freq");
      a.w_o = lt.at("attn.w_o");
    }
    if (L.has_lin) {
      Linear &l = L.lin;
      l.q_off = num("lin.q_off");
      l.k_off = num("lin.k_off");
      l.v_off = num("lin.v_off");
      l.g_off = num("lin.g_off");
      l.H = num("lin.heads");
      l.V = num("lin.vdim");
      l.act = num("lin.act");
      l.gate_act = num("lin.gate_act");
      l.groups = num("lin.groups");
      l.state = num("lin.state");
      l.qscale = num("lin.qscale");
      l.out_scale = num("lin.out_scale");
      l.channel = num("lin.channel") != 0;
      l.w_o = lt.at("lin.w_o");
      l.norm = lt.at("lin.norm");
      l.decay = ten("lin.decay");
      l.powers = ten("lin.powers");
      if (l.channel) {
        l.a_off = num("lin.a_off");
        l.tau = num("lin.tau");
        l.a2 = lt.at("lin.a2");
        l.a2_b = lt.at("lin.a2_b");
      }
    }
    if (L.has_mlp) {
      L.gate_up = lt.at("gate_up");
      L.down = lt.at("down");
      L.norm2 = lt.at("norm2");
    }
    m.layers.push_back(std::move(L));
  }
  registry()[key] = std::move(m);
}

inline const Model &find(const std::string &key) {
  auto it = registry().find(key);
  TORCH_CHECK(it != registry().end(), "model not registered: ", key);
  return it->second;
}

// One batch: decode rows 0..n_decode-1 (one per sequence, in the order of the
// first rows of block_tables / state_slots), then prefill rows.
struct Batch {
  const Tensors &t;
  int64_t n_decode, max_ctx, max_kv, rows;
  const Tensor &at(const char *k) const { return t.at(k); }
  bool prefill() const { return rows > n_decode; }
};

inline Tensor attention(const Model &m, const Attn &a, const Batch &b,
                        const Tensor &proj, Tensor kc, Tensor vc) {
  auto q = torch::empty({b.rows, a.H, a.D}, proj.options());
  auto out = torch::empty_like(q);
  const Tensor &bt = b.at("block_tables");
  qk_norm_rope_store(q, kc, vc, proj, a.q_off, a.k_off, a.q_norm, a.k_norm,
                     b.at("positions"), b.at("slots"), a.freq, a.mag, m.eps);
  if (!attn_tiles_ok(q) || a.H / kc.size(1) > 16) {
    local_attn_rows(out, q, kc, vc, bt, b.at("row_seq"), b.at("positions"),
                    a.scale, a.chunk, a.sink);
  } else {
    if (b.n_decode)
      local_attn_decode(out, q, kc, vc, bt, b.at("ctx_lens"), a.scale,
                        a.chunk, a.sink, b.max_ctx);
    if (b.prefill())
      local_attn_prefill(out, q, kc, vc, bt, b.at("tile_q0"),
                         b.at("tile_qn"), b.at("tile_seq"),
                         b.at("tile_pos0"), a.scale, a.chunk, a.sink,
                         b.max_kv);
  }
  return at::linear(out.view({b.rows, a.H * a.D}), a.w_o);
}

inline Tensor linear_mixer(const Model &m, const Linear &l, const Batch &b,
                           const Tensor &proj, Tensor state) {
  auto o = torch::empty({b.rows, l.H * l.V}, proj.options());
  const Tensor &slots = b.at("state_slots");
  const Tensor &positions = b.at("positions");
  const bool tiles = linear_tiles_ok(proj, state);
  Tensor ld;
  if (l.channel) {
    ld = torch::empty({b.rows, l.a2.size(0)},
                      proj.options().dtype(torch::kFloat32));
    const int64_t alone = tiles ? b.n_decode : b.rows;
    log_decay(ld, proj, l.a_off, l.a2, l.a2_b, l.tau, 0, alone, c10::nullopt,
              c10::nullopt);
    if (tiles && b.prefill())
      log_decay(ld, proj, l.a_off, l.a2, l.a2_b, l.tau, 0, 0,
                b.at("chunk_row0"), b.at("chunk_len"));
  }
  if (b.n_decode)
    linear_recurrent(o, proj, l.q_off, l.k_off, l.v_off, l.act, l.qscale,
                     l.channel ? ld : l.decay, l.channel, state, c10::nullopt,
                     c10::nullopt, slots.narrow(0, 0, b.n_decode), positions);
  if (b.prefill()) {
    auto seg_slot = slots.narrow(0, b.n_decode, slots.size(0) - b.n_decode);
    if (tiles)
      linear_chunked(o, proj, l.q_off, l.k_off, l.v_off, l.act, l.qscale,
                     l.channel ? ld : l.powers, l.channel, state,
                     b.at("chunk_row0"), b.at("chunk_len"), b.at("seg_row0"),
                     b.at("seg_chunk0"), seg_slot, positions);
    else
      linear_recurrent(o, proj, l.q_off, l.k_off, l.v_off, l.act, l.qscale,
                       l.channel ? ld : l.decay, l.channel, state,
                       b.at("seg_row0"), b.at("seg_len"), seg_slot,
                       positions);
  }
  auto gated = torch::empty_like(o);
  gated_norm(gated, o, proj, l.g_off, l.norm, l.groups, l.gate_act, m.eps);
  return at::linear(gated, l.w_o);
}

inline Tensor forward(const std::string &key, const Tensors &tensors,
                      int64_t n_decode, int64_t max_ctx, int64_t max_kv,
                      std::vector<Tensor> kcaches,
                      std::vector<Tensor> vcaches,
                      std::vector<Tensor> states) {
  const Model &m = find(key);
  const Tensor &tokens = tensors.at("tokens");
  const Batch b{tensors, n_decode, max_ctx, max_kv, tokens.size(0)};
  const int64_t width = m.embed.size(1);
  auto x = torch::empty({b.rows, width},
                        m.embed.options().dtype(torch::kFloat32));
  auto h = torch::empty({b.rows, width}, m.embed.options());
  embed_positions(x, h, m.embed,
                  m.pos.defined() ? OptTensor(m.pos) : c10::nullopt, tokens,
                  b.at("positions"));
  for (const Layer &L : m.layers) {
    auto proj = at::linear(h, L.w_in);
    Tensor first, second;
    double s1 = 1.0, s2 = 0.0;
    if (L.has_attn) {
      first = attention(m, L.attn, b, proj, kcaches.at(L.attn.cache),
                        vcaches.at(L.attn.cache));
      s1 = L.attn.out_scale;
    }
    if (L.has_lin) {
      auto y = linear_mixer(m, L.lin, b, proj, states.at(L.lin.state));
      if (first.defined()) { second = y; s2 = L.lin.out_scale; }
      else { first = y; s1 = L.lin.out_scale; }
    }
    post_norm(x, h, first, s1,
              second.defined() ? OptTensor(second) : c10::nullopt, s2,
              m.alpha, L.norm1, m.eps);
    if (L.has_mlp) {
      auto gu = at::linear(h, L.gate_up);
      auto act = torch::empty({b.rows, gu.size(1) / 2}, gu.options());
      glu(act, gu);
      post_norm(x, h, at::linear(act, L.down), 1.0, c10::nullopt, 0.0,
                m.alpha, L.norm2, m.eps);
    }
  }
  return x;
}

inline Tensor compute_logits(const std::string &key, Tensor x, Tensor rows) {
  const Model &m = find(key);
  auto h = torch::empty({rows.size(0), x.size(1)}, m.head.options());
  norm_rows(h, x, rows, m.final_norm, m.eps);
  return at::linear(h, m.head).to(torch::kFloat32);
}

inline void unregister_model(const std::string &key) {
  registry().erase(key);
}

}  // namespace qhybrid
