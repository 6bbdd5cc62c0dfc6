// Blocks of the recurrent and chunk-local models: a mixer that may hold a
// chunk-local attention part ("attn.*") and a linear-attention part ("lin.*"),
// both reading the rows of one fused input projection `w_in`, each with its
// own output projection, joined with their scales by the norm after the sum;
// and the gated feed-forward.
//
// Included by hybrid_bindings.cpp after the kernel wrappers it calls.
#pragma once

namespace qhybrid {

struct Attn {
  int64_t q_off, k_off, H, D, chunk;
  double scale, mag, out_scale;
  bool sink;
  Tensor q_norm, k_norm, freq, w_o;

  Attn(const Tensors &t, const Numbers &n)
      : q_off(n.at("attn.q_off")), k_off(n.at("attn.k_off")),
        H(n.at("attn.heads")), D(n.at("attn.dim")), chunk(n.at("attn.chunk")),
        scale(n.at("attn.scale")), mag(n.at("attn.mag")),
        out_scale(n.at("attn.out_scale")), sink(n.at("attn.sink") != 0),
        q_norm(t.at("attn.q_norm")), k_norm(t.at("attn.k_norm")),
        freq(t.at("attn.freq")), w_o(t.at("attn.w_o")) {}
};

struct Linear {
  int64_t q_off, k_off, v_off, g_off, a_off = 0, H, V, act, gate_act, groups;
  double qscale, tau = 1.0, out_scale;
  bool channel;                 // decay per key channel and token
  Tensor w_o, norm;
  Tensor decay, powers;         // one constant per head
  Tensor a2, a2_b;              // channel: low-rank decay

  Linear(const Tensors &t, const Numbers &n)
      : q_off(n.at("lin.q_off")), k_off(n.at("lin.k_off")),
        v_off(n.at("lin.v_off")), g_off(n.at("lin.g_off")),
        H(n.at("lin.heads")), V(n.at("lin.vdim")), act(n.at("lin.act")),
        gate_act(n.at("lin.gate_act")), groups(n.at("lin.groups")),
        qscale(n.at("lin.qscale")), out_scale(n.at("lin.out_scale")),
        channel(n.at("lin.channel") != 0), w_o(t.at("lin.w_o")),
        norm(t.at("lin.norm")), decay(find_or_none(t, "lin.decay")),
        powers(find_or_none(t, "lin.powers")) {
    if (channel) {
      a_off = n.at("lin.a_off");
      tau = n.at("lin.tau");
      a2 = t.at("lin.a2");
      a2_b = t.at("lin.a2_b");
    }
  }
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

struct MixerBlock : Block {
  Tensor w_in, norm;
  std::unique_ptr<Attn> attn;
  std::unique_ptr<Linear> lin;

  void run(const Model &m, const Run &r, const Batch &b, const Pools &pools,
           Stream &s, const Next &) const override {
    auto proj = at::linear(s.h, w_in);
    Tensor first, second;
    double s1 = 1.0, s2 = 0.0;
    if (attn) {
      first = attention(m, *attn, b, proj, pools.at("k").at(r.attn),
                        pools.at("v").at(r.attn));
      s1 = attn->out_scale;
    }
    if (lin) {
      auto y = linear_mixer(m, *lin, b, proj, pools.at("state").at(r.state));
      if (first.defined()) { second = y; s2 = lin->out_scale; }
      else { first = y; s1 = lin->out_scale; }
    }
    post_norm(s.x, s.h, first, s1, opt(second), s2, m.alpha, norm, m.eps);
  }
};

struct GluBlock : Block {
  Tensor gate_up, down, norm;

  void run(const Model &m, const Run &, const Batch &b, const Pools &,
           Stream &s, const Next &) const override {
    auto gu = at::linear(s.h, gate_up);
    auto act = torch::empty({b.rows, gu.size(1) / 2}, gu.options());
    glu(act, gu);
    post_norm(s.x, s.h, at::linear(act, down), 1.0, c10::nullopt, 0.0,
              m.alpha, norm, m.eps);
  }
};

Layer make_layer(const Tensors &t, const Numbers &n) {
  Layer blocks;
  const bool has_attn = t.count("attn.w_o"), has_lin = t.count("lin.w_o");
  if (!has_attn && !has_lin) return blocks;
  auto mixer = std::make_shared<MixerBlock>();
  mixer->w_in = t.at("w_in");
  mixer->norm = t.at("norm1");
  if (has_attn) mixer->attn = std::make_unique<Attn>(t, n);
  if (has_lin) mixer->lin = std::make_unique<Linear>(t, n);
  blocks.push_back(mixer);
  if (t.count("gate_up")) {
    auto ff = std::make_shared<GluBlock>();
    ff->gate_up = t.at("gate_up");
    ff->down = t.at("down");
    ff->norm = t.at("norm2");
    blocks.push_back(ff);
  }
  return blocks;
}

}  // namespace qhybrid
