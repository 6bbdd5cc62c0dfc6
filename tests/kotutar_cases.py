"""Small Kotutar configurations with random weights."""

import math

import torch

import hybrid_cases
import kotutar_oracle as oracle


def mixer(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
            "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
            "rot": {"dims": rot_dim, "base": base}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top},
           "expert": {"ff": ff}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def config(vocab, width, eps, loop, *layers):
    return {"architecture": "Kotutar", "vocab": vocab, "width": width,
            "norm": {"eps": eps}, "loop": loop,
            "layers": [{"type": "latent_attention", "mixer": m, "mlp": f}
                       for m, f in layers]}


# name -> configuration; sizes are chosen so that nothing is equal by chance
CONFIGS = {
    # the matrix-core paths, in the latent space and expanded; mixers differ
    # from layer to layer, one layer has no feed-forward
    "tiles": config(
        300, 80, 3e-5, {"start": 1, "stop": 3, "times": 3},
        (mixer(5, 24, 16, 40, 48, 72, 0.21, 5000.0), dense(104)),
        (mixer(3, 40, 8, 24, 64, 64, 0.3, 300.0), moe(7, 2, 56, 88)),
        (mixer(8, 16, 32, 16, 40, 48, 0.17, 1e5), None),
        (mixer(2, 64, 24, 72, 56, 104, 0.1, 800.0), moe(5, 1, 40))),
    # sizes no vector load takes, every expert chosen, no pass repeated
    "odd": config(
        271, 54, 1e-6, None,
        (mixer(3, 10, 6, 13, 21, 19, 0.35, 900.0), moe(3, 3, 33, 17)),
        (mixer(1, 7, 2, 11, 9, 5, 0.6, 50.0), dense(70))),
    # one head, one expert, one pass; the latent is smaller than the heads,
    # so short prompts are never expanded
    "small": config(
        290, 40, 1e-4, {"start": 0, "stop": 1, "times": 1},
        (mixer(1, 16, 2, 16, 8, 8, 0.22, 77.0), moe(1, 1, 24)),
        (mixer(2, 32, 16, 64, 24, 16, 0.2, 1e4), dense(56))),
    # many heads and experts, the largest head sizes of the prefill tiles, the
    # last layer is part of the loop
    "wide": config(
        280, 136, 1e-5, {"start": 1, "stop": 2, "times": 2},
        (mixer(18, 64, 64, 128, 72, 136, 0.09, 1e4), dense(48)),
        (mixer(2, 192, 64, 248, 96, 264, 0.06, 2e4), moe(70, 3, 48, 64))),
    # a latent and a rotated part that no matrix kernel takes, beside a layer
    # that one does
    "mixed": config(
        275, 48, 2e-5, {"start": 0, "stop": 2, "times": 2},
        (mixer(2, 16, 72, 24, 32, 520, 0.1, 3e3), dense(40)),
        (mixer(4, 32, 8, 32, 40, 56, 0.16, 1e3), moe(4, 2, 40, 24))),
}
STEP = 1.5                  # stream of a token's chosen experts, per rank


def random_weights(cfg, seed=0):
    """{name: tensor} in bf16-exact values, large enough that every branch
    moves the logits.

    The routers' choices must not be close calls, or rounding would turn
    them: the first stream columns, one per expert of every router, hold a
    pattern that only depends on the token (its own expert highest, the next
    ones in steps below it), the sublayers leave them almost alone, and a
    router's rows read its columns."""
    g = torch.Generator().manual_seed(seed)

    def mat(o, i, gain=1.0):
        return torch.randn(o, i, generator=g) * gain / math.sqrt(i)

    def norm(n, lo=0.6, span=0.8):
        return lo + span * torch.rand(n, generator=g)

    w, V = cfg["width"], cfg["vocab"]
    first, E = {}, 0                     # layer -> its experts' columns
    t = {"embed": mat(V, w, math.sqrt(w))}
    for i, layer in enumerate(cfg["layers"]):
        if not layer["mlp"] or layer["mlp"]["kind"] != "moe":
            continue
        r = layer["mlp"]["router"]
        n, top = r["experts"], r["top"]
        first[i], E = E, E + n
        t["embed"][:, first[i]:E] = 0.0
        for tok in range(V):
            for k in range(min(top + 1, n)):
                t["embed"][tok, first[i] + (tok * 3 + k) % n] = \
                    STEP * (top + 1 - k)
    if cfg["loop"]:
        t["loop.in"] = mat(w, 2 * w)
        t["loop.in"][:E] = 0.0
        for e in range(E):
            t["loop.in"][e, e], t["loop.in"][e, w + e] = 0.625, 0.375
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        names = ["norm1", "norm1b"] + (["norm2", "norm2b"] if f else [])
        for n in names:
            t[p + n] = norm(w)
            if n.endswith("b"):
                t[p + n][:E] = 0.01
        q = p + "mix."
        H, D, R = m["heads"], m["dim"], m["rot_dim"]
        t.update({q + "dq": mat(m["q_rank"], w),
                  q + "dq.norm": norm(m["q_rank"]),
                  q + "uq": mat(H * (D + R), m["q_rank"], 1.5),
                  q + "dkv": mat(m["kv_rank"] + R, w),
                  q + "dkv.norm": norm(m["kv_rank"]),
                  q + "uk": mat(H * D, m["kv_rank"], 1.5),
                  q + "uv": mat(H * m["vdim"], m["kv_rank"]),
                  q + "sink": 1.0 + torch.randn(H, generator=g),
                  q + "o": mat(w, H * m["vdim"], 1.5)})
        if f is None:
            continue
        q = p + "mlp."
        if f["kind"] == "dense":
            ff = f["ff"]
            t.update({q + "up": mat(ff, w),
                      q + "up.b": 0.5 * torch.randn(ff, generator=g),
                      q + "down": mat(w, ff),
                      q + "down.b": 0.3 * torch.randn(w, generator=g)})
            continue
        n, ff = f["router"]["experts"], f["expert"]["ff"]
        t[q + "router"] = mat(n, w, 0.02)
        cols = [first[i] + e for e in range(n)]
        t[q + "router"][range(n), cols] = 0.5
        t[p + "norm2"][cols] = 1.0
        for e in range(n):
            t.update({f"{q}e{e}.up": mat(ff, w, 1.5),
                      f"{q}e{e}.down": mat(w, ff, 1.5)})
        if f.get("shared"):
            ff = f["shared"]["ff"]
            t.update({q + "shared.up": mat(ff, w),
                      q + "shared.down": mat(w, ff),
                      q + "shared.sg": mat(1, w)})
    t["final.norm"] = norm(w)
    t["head"] = mat(V, w)
    t["head"][:, :E] *= 0.1
    return {k: v.to(torch.bfloat16) for k, v in t.items()}


class Case(hybrid_cases.Case):
    def __init__(self, name, folder, cfg=None, seed=0):
        cfg = cfg or CONFIGS[name]
        super().__init__(name, folder, cfg, random_weights(cfg, seed), oracle)
