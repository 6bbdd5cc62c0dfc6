"""Small Koridra configurations with random weights, and helpers that feed
them to the engine and to the plain oracle."""

import json
import math
import os
import struct

import torch

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


def write_checkpoint(folder, cfg, weights):
    """config.json + model.safetensors."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name, w in weights.items():
        raw = w.contiguous().view(torch.int16).numpy().tobytes()
        header[name] = {"dtype": "BF16", "shape": list(w.shape),
                        "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + b"".join(blobs))
    return folder


def tokens_for(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,),
                         generator=torch.Generator().manual_seed(seed)).tolist()


class Case:
    """One configuration on disk, its weights, and remembered oracle logits."""

    def __init__(self, name, folder, cfg=None, seed=0):
        self.name = name
        self.cfg = cfg or CONFIGS[name]
        self.weights = random_weights(self.cfg, RANKS.get(name, 4), seed)
        self.path = write_checkpoint(str(folder), self.cfg, self.weights)
        self._known = {}

    def logits(self, tokens):
        key = tuple(tokens)
        if key not in self._known:
            self._known[key] = oracle.forward(self.cfg, self.weights,
                                              tokens)[0]
        return self._known[key]

    def engine(self, device, dtype, blocks=96, slots=4, **kw):
        from quoracle_amd.engine.engine import LocalEngine
        return LocalEngine([self.path], device=torch.device(device),
                           embed_model_key=None, kv_blocks_override=blocks,
                           dtype=dtype, state_slots=slots, **kw)


def error(got, want):
    """Largest per-row RMS difference, in units of the logits' RMS."""
    got, want = got.double(), want.double()
    d = (got - want).square().mean(-1).sqrt()
    return float(d.max() / want.square().mean().sqrt())


def tolerance(dtype):
    return 2e-5 if dtype == torch.float32 else 0.06


def feed(engine, path, schedule):
    """Run [[(id, tokens), ...], ...] with every place wanted; returns
    {id: logits of all its tokens so far}.  A request ends when its id is
    given as (id, None)."""
    out, live = {}, set()
    for step in schedule:
        ends = [i for i, toks in step if toks is None]
        parts = [(i, toks) for i, toks in step if toks]
        live.update(i for i, _ in parts)
        if parts:
            lg = engine.step_entries(
                path, [(i, toks, range(len(toks))) for i, toks in parts],
                live)
            at = 0
            for i, toks in parts:
                out.setdefault(i, []).append(lg[at:at + len(toks)])
                at += len(toks)
        for i in ends:
            engine.drop_session(path, i)
            live.discard(i)
    return {i: torch.cat(p) for i, p in out.items()}


def cut(tokens, sizes):
    """Split tokens into portions of the given sizes, cycling."""
    parts, at, k = [], 0, 0
    while at < len(tokens):
        n = sizes[k % len(sizes)]
        parts.append(tokens[at:at + n])
        at, k = at + n, k + 1
    return parts


