// Native layer loop of the hybrid models.
//
// A model is a list of layer runs over a list of layers; a layer is a list of
// blocks (a mixer or a feed-forward, with its residual sum and norms), made by
// the module's make_layer() from a map of tensors and a map of numbers.  Plain
// matrix products go to the vendor library.
//
// Included after hybrid_host.h; the module defines make_layer().
#pragma once

#include <map>
#include <memory>
#include <unordered_map>
#include <vector>

namespace qhybrid {

using Tensors = std::map<std::string, Tensor>;
using Numbers = std::map<std::string, double>;
using Counts = std::map<std::string, int64_t>;
using Pools = std::map<std::string, std::vector<Tensor>>;

// One batch: decode rows 0..n_decode-1 (one per sequence, in the order of the
// first rows of block_tables / state_slots), then prefill rows.
struct Batch {
  const Tensors &t;
  int64_t n_decode, n_latent, max_ctx, max_kv, rows;
  const Tensor &at(const char *k) const { return t.at(k); }
  bool has(const char *k) const {
    auto it = t.find(k);
    return it != t.end() && it->second.numel() > 0;
  }
  bool prefill() const { return rows > n_decode; }
};

inline Batch make_batch(const Tensors &t, const Counts &n, int64_t rows) {
  return Batch{t, n.at("n_decode"), n.at("n_latent"), n.at("max_ctx"),
               n.at("max_kv"), rows};
}

// One run of a layer: where it finds its cache and state.
struct Run {
  int64_t layer, attn, state, latent;
  bool enter;                   // the embedding output joins before it
};

struct Stream {
  Tensor x;                     // float32 residual
  Tensor h;                     // what the next block reads
  Tensor joined;                // [x, embedding output] of looped models
};

// What the stream goes through behind a block: the next block's norm, or the
// first half of `joined`.
struct Next {
  Tensor norm;
  bool join = false;
};

struct Model;

struct Block {
  Tensor pre;                   // norm of the block's input; undefined: none
  virtual ~Block() = default;
  virtual void run(const Model &m, const Run &r, const Batch &b,
                   const Pools &pools, Stream &s, const Next &next) const = 0;
};

using Layer = std::vector<std::shared_ptr<Block>>;

struct Model {
  Tensor embed, pos, head, final_norm, loop_in;
  double alpha, eps;
  std::vector<Layer> layers;
  std::vector<Run> runs;
};

// From the module.
Layer make_layer(const Tensors &t, const Numbers &n);

inline Tensor find_or_none(const Tensors &t, const char *k) {
  auto it = t.find(k);
  return it == t.end() ? Tensor() : it->second;
}

inline OptTensor opt(const Tensor &t) {
  return t.defined() ? OptTensor(t) : c10::nullopt;
}

inline std::unordered_map<std::string, Model> &registry() {
  static std::unordered_map<std::string, Model> models;
  return models;
}

inline void register_model(const std::string &key, const Tensors &t,
                           const Numbers &n,
                           const std::vector<Tensors> &layer_tensors,
                           const std::vector<Numbers> &layer_numbers,
                           const std::vector<Counts> &runs) {
  Model m;
  m.embed = t.at("embed");
  m.pos = find_or_none(t, "pos");
  m.loop_in = find_or_none(t, "loop_in");
  m.head = t.at("head");
  m.final_norm = t.at("final_norm");
  m.alpha = n.at("alpha");
  m.eps = n.at("eps");
  TORCH_CHECK(layer_tensors.size() == layer_numbers.size(), "layers");
  for (size_t i = 0; i < layer_tensors.size(); ++i) {
    m.layers.push_back(make_layer(layer_tensors[i], layer_numbers[i]));
    TORCH_CHECK(!m.layers.back().empty(), "layer without a mixer");
  }
  for (const Counts &r : runs) {
    m.runs.push_back(Run{r.at("layer"), r.at("attn"), r.at("state"),
                         r.at("latent"), r.at("enter") != 0});
    TORCH_CHECK(m.runs.back().layer < (int64_t)m.layers.size(), "run");
    TORCH_CHECK(!m.runs.back().enter || m.loop_in.defined(), "loop_in");
  }
  registry()[key] = std::move(m);
}

inline const Model &find(const std::string &key) {
  auto it = registry().find(key);
  TORCH_CHECK(it != registry().end(), "model not registered: ", key);
  return it->second;
}

inline Tensor forward(const std::string &key, const Tensors &tensors,
                      const Counts &counts, const Pools &pools) {
  const Model &m = find(key);
  const Tensor &tokens = tensors.at("tokens");
  const Batch b = make_batch(tensors, counts, tokens.size(0));
  const int64_t width = m.embed.size(1);
  Stream s;
  s.x = torch::empty({b.rows, width},
                     m.embed.options().dtype(torch::kFloat32));
  s.h = torch::empty({b.rows, width}, m.embed.options());
  embed_positions(s.x, s.h, m.embed, opt(m.pos), tokens, b.at("positions"));
  if (m.loop_in.defined()) s.joined = at::cat({s.h, s.h}, 1);
  for (size_t i = 0; i < m.runs.size(); ++i) {
    const Run &r = m.runs[i];
    const Layer &blocks = m.layers[r.layer];
    if (r.enter)
      pre_norm(s.x, s.h, linear_f32(s.joined, m.loop_in), blocks[0]->pre,
               m.eps);
    else if (i == 0 && blocks[0]->pre.defined())
      pre_norm(s.x, s.h, c10::nullopt, blocks[0]->pre, m.eps);
    for (size_t k = 0; k < blocks.size(); ++k) {
      Next next;
      if (k + 1 < blocks.size()) {
        next.norm = blocks[k + 1]->pre;
      } else if (i + 1 < m.runs.size()) {
        next.join = m.runs[i + 1].enter;
        if (!next.join) next.norm = m.layers[m.runs[i + 1].layer][0]->pre;
      }
      blocks[k]->run(m, r, b, pools, s, next);
    }
  }
  return s.x;
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

inline void bind(pybind11::module_ &m) {
  m.def("embed_positions", &embed_positions,
        "Token embedding plus learned positions into the float32 stream");
  m.def("norm_rows", &norm_rows, "Final RMS norm of selected rows");
  m.def("pre_norm", &pre_norm, "RMS norm of the float32 stream");
  m.def("register_model", &register_model,
        "Register a model's weights with the native driver");
  m.def("unregister_model", &unregister_model, "Drop a registered model");
  m.def("forward", &forward,
        "All layer runs of one mixed batch; returns the float32 stream");
  m.def("logits", &compute_logits, "Final norm and head of selected rows");
}

}  // namespace qhybrid
