"""Small Koridra configurations with random weights."""

import math

import torch

import hybrid_cases
import koridra_oracle as oracle

# name -> configuration; sizes are chosen so that nothing is equal by chance
CONFIGS = {
    # vector-friendly head sizes: the matrix-core paths on the GPU
    "tiles": {
        "architecture": "Koridra", "vocab": 300, "width": 80,
        "max_positions": 700, "postln_alpha": 1.7, "norm": {"eps": 3e-5},
        "layers": [
            {"type": "parallel", "mlp": {"kind": "dense", "ff": 104},
             "mixer": {
                 "left": {"heads": 6, "kv_heads": 2, "dim": 40, "vdim": 40,
                          "scale": 0.21, "mask": {"size": 37},
                          "rot": {"dims": 16, "base": 5000.0, "scaling": {
                              "factor": 3.0, "original": 64, "fast": 8.0,
                              "slow": 1.0}}},
                 "right": {"heads": 3, "dim": 24, "vdim": 72, "tau": 5.0},
                 "left_scale": 0.6, "right_scale": 1.3}},
            {"type": "lightning", "mlp": None,
             "mixer": {"heads": 4, "dim": 16, "vdim": 40,
                       "decay": [1.0, 0.97, 0.6, 0.03]}},
            {"type": "lightning", "mlp": {"kind": "dense", "ff": 64},
             "mixer": {"heads": 2, "dim": 72, "vdim": 24,
                       "decay": [0.999, 0.8]}},
        ]},
    # head sizes no vector load takes, no frequency scaling
    "odd": {
        "architecture": "Koridra", "vocab": 271, "width": 54,
        "max_positions": 650, "postln_alpha": 0.9, "norm": {"eps": 1e-6},
        "layers": [
            {"type": "lightning", "mlp": {"kind": "dense", "ff": 70},
             "mixer": {"heads": 3, "dim": 10, "vdim": 13,
                       "decay": [0.5, 0.9, 0.995]}},
            {"type": "parallel", "mlp": {"kind": "dense", "ff": 33},
             "mixer": {
                 "left": {"heads": 3, "kv_heads": 3, "dim": 18, "vdim": 18,
                          "scale": 0.3, "mask": {"size": 50},
                          "rot": {"dims": 6, "base": 900.0}},
                 "right": {"heads": 5, "dim": 7, "vdim": 11, "tau": 1.0},
                 "left_scale": 1.1, "right_scale": -0.4}},
        ]},
    # many query heads on one key head, large key dims, two mixed layers
    "wide": {
        "architecture": "Koridra", "vocab": 290, "width": 96,
        "max_positions": 600, "postln_alpha": 2.2, "norm": {"eps": 1e-5},
        "layers": [
            {"type": "parallel", "mlp": {"kind": "dense", "ff": 48},
             "mixer": {
                 "left": {"heads": 18, "kv_heads": 1, "dim": 16, "vdim": 16,
                          "scale": 0.25, "mask": {"size": 64},
                          "rot": {"dims": 16, "base": 10000.0, "scaling": {
                              "factor": 8.0, "original": 128, "fast": 16.0,
                              "slow": 2.0}}},
                 "right": {"heads": 1, "dim": 136, "vdim": 8, "tau": 16.0},
                 "left_scale": 1.0, "right_scale": 1.0}},
            {"type": "parallel", "mlp": None,
             "mixer": {
                 "left": {"heads": 2, "kv_heads": 1, "dim": 128, "vdim": 128,
                          "scale": 0.09, "mask": {"size": 1},
                          "rot": {"dims": 128, "base": 700.0}},
                 "right": {"heads": 2, "dim": 32, "vdim": 96, "tau": 2.0},
                 "left_scale": 0.5, "right_scale": 0.8}},
        ]},
    # no attention at all: no pages' bytes, only states
    "recurrent": {
        "architecture": "Koridra", "vocab": 280, "width": 40,
        "max_positions": 400, "postln_alpha": 1.2, "norm": {"eps": 1e-4},
        "layers": [
            {"type": "lightning", "mlp": {"kind": "dense", "ff": 56},
             "mixer": {"heads": 1, "dim": 48, "vdim": 136,
                       "decay": [0.98]}}]},
}
RANKS = {"tiles": 4, "odd": 3, "wide": 21}


def random_weights(cfg, rank, seed=0):
    """{name: tensor} in bf16-exact values, large enough that every branch
    moves the logits."""
    g = torch.Generator().manual_seed(seed)

    def mat(o, i, gain=1.0):
        return torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def norm(n):
        return 0.6 + 0.8 * torch.rand(n, generator=g)

    w, V = cfg["width"], cfg["vocab"]
    t = {"embed": mat(V, w, math.sqrt(w)),
         "pos": 0.3 * torch.randn(cfg["max_positions"], w, generator=g)}

    def linear(p, m, channel):
        kd, vd = m["heads"] * m["dim"], m["heads"] * m["vdim"]
        t.update({p + "q": mat(kd, w), p + "k": mat(kd, w),
                  p + "v": mat(vd, w), p + "g": mat(vd, w),
                  p + "o": mat(w, vd, 1.5),
                  p + "norm": norm(m["vdim"] if channel else vd)})
        if channel:
            t.update({p + "a1": mat(rank, w), p + "a2": mat(kd, rank, 2.0),
                      p + "a2.b": 2.0 * torch.randn(kd, generator=g)})

    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        t[p + "norm1"] = norm(w)
        if layer["type"] == "lightning":
            linear(p + "mix.", m, False)
        else:
            a, q = m["left"], p + "mix.left."
            nq, nk = a["heads"] * a["dim"], a["kv_heads"] * a["dim"]
            t.update({q + "q": mat(nq, w), q + "k": mat(nk, w),
                      q + "q.norm": 1.5 * norm(nq),
                      q + "k.norm": 1.5 * norm(nk), q + "o": mat(w, nq, 2.0)})
            linear(p + "mix.right.", m["right"], True)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            t.update({p + "mlp.gate": mat(ff, w), p + "mlp.up": mat(ff, w),
                      p + "mlp.down": mat(w, ff, 2.0), p + "norm2": norm(w)})
    t["final.norm"] = norm(w)
    t["head"] = mat(V, w)
    return {k: v.to(torch.bfloat16) for k, v in t.items()}


class Case(hybrid_cases.Case):
    def __init__(self, name, folder, cfg=None, seed=0):
        cfg = cfg or CONFIGS[name]
        super().__init__(name, folder, cfg,
                         random_weights(cfg, RANKS.get(name, 4), seed), oracle)
