"""Plain, slow Kotutar in float64: one function per mechanism.

Token by token and key by key, straight from the equations, over a dict of
named weight matrices ([out, in], applied as W x) and the plain configuration
dict.  Nothing here is shared with quoracle_amd: it is what the framework's
kernels, cache and scheduler are compared against.
"""

import math

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def gelu(z):
    """The exact form: z times the normal distribution function."""
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def rotate(x, position, dims, base):
    """Turn the pairs (2i, 2i+1), i < dims / 2, of the last axis by
    position * base^(-2i/dims); what lies behind them passes."""
    y = x.clone()
    for i in range(dims // 2):
        a = position * base ** (-2.0 * i / dims)
        c, s = math.cos(a), math.sin(a)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * c - v * s
        y[..., 2 * i + 1] = v * c + u * s
    return y


def sees(i, j):
    return j <= i


def sink_softmax(scores, sink):
    """Weights of the scores [n, H] over n when exp(sink) [H] joins the
    denominator."""
    top = torch.maximum(scores.max(0).values, sink)
    e = torch.exp(scores - top)
    return e / (torch.exp(sink - top) + e.sum(0))


def attend(q, keys, values, scale, sink, positions=None):
    """q [Tq, H, D] at `positions` (default 0..) over keys [T, H, D] and
    values [T, H, V]; sink [H]."""
    positions = range(q.shape[0]) if positions is None else positions
    out = torch.zeros(q.shape[0], q.shape[1], values.shape[2], dtype=q.dtype)
    for r, i in enumerate(positions):
        js = [j for j in range(keys.shape[0]) if sees(i, j)]
        w = sink_softmax((keys[js] * q[r]).sum(-1) * scale, sink)
        out[r] = (w[:, :, None] * values[js]).sum(0)
    return out


def latent_of(h, W, p, m, eps, positions=None):
    """(c [T, kv_rank], rotated key part [T, rot_dim]): what a cache holds."""
    R, n = m["kv_rank"], m["rot_dim"]
    positions = range(h.shape[0]) if positions is None else positions
    both = h @ W[p + "dkv"].T
    c = rms_norm(both[:, :R], W[p + "dkv.norm"], eps)
    k = torch.stack([rotate(both[t, R:R + n], i, n, m["rot"]["base"])
                     for t, i in enumerate(positions)])
    return c, k


def latent_queries(h, W, p, m, eps, positions=None):
    """[T, H, dim + rot_dim], the rotated part last."""
    T, H, D, n = h.shape[0], m["heads"], m["dim"], m["rot_dim"]
    positions = range(T) if positions is None else positions
    q = rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], eps) @ W[p + "uq"].T
    q = q.view(T, H, D + n).clone()
    for t, i in enumerate(positions):
        q[t, :, D:] = rotate(q[t, :, D:], i, n, m["rot"]["base"])
    return q


def latent_attention(h, W, p, m, eps):
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    c, k_rot = latent_of(h, W, p, m, eps)
    q = latent_queries(h, W, p, m, eps)
    k = torch.cat([(c @ W[p + "uk"].T).view(T, H, D),
                   k_rot[:, None, :].expand(T, H, k_rot.shape[1])], -1)
    v = (c @ W[p + "uv"].T).view(T, H, V)
    o = attend(q, k, v, m["scale"], W[p + "sink"])
    return o.reshape(T, H * V) @ W[p + "o"].T


MIXERS = {"latent_attention": latent_attention}


def dense_ff(h, W, p, m):
    return gelu(h @ W[p + "up"].T + W[p + "up.b"]) @ W[p + "down"].T \
        + W[p + "down.b"]


def expert(h, W, p):
    return gelu(h @ W[p + "up"].T) @ W[p + "down"].T


def route(h, W, p, router):
    """[(expert, weight), ...] of each token."""
    s = torch.sigmoid(h @ W[p + "router"].T)
    picks = []
    for row in s:
        order = sorted(range(router["experts"]), key=lambda e: -float(row[e]))
        picks.append([(e, row[e]) for e in order[:router["top"]]])
    return picks


def moe_ff(h, W, p, m):
    out = torch.zeros_like(h)
    for t, picks in enumerate(route(h, W, p, m["router"])):
        for e, w in picks:
            out[t] = out[t] + expert(w * h[t], W, f"{p}e{e}.")
    if m.get("shared"):
        gate = torch.sigmoid(h @ W[p + "shared.sg"].T)
        out = out + gate * expert(h, W, p + "shared.")
    return out


FEED_FORWARD = {"dense": dense_ff, "moe": moe_ff}


def layer(x, W, i, spec, eps):
    p = f"l{i}."
    y = MIXERS[spec["type"]](rms_norm(x, W[p + "norm1"], eps), W, p + "mix.",
                             spec["mixer"], eps)
    x = x + rms_norm(y, W[p + "norm1b"], eps)
    if spec["mlp"] is not None:
        y = FEED_FORWARD[spec["mlp"]["kind"]](
            rms_norm(x, W[p + "norm2"], eps), W, p + "mlp.", spec["mlp"])
        x = x + rms_norm(y, W[p + "norm2b"], eps)
    return x


def passes(cfg):
    """[(layers of the pass, does the embedding join before it), ...]."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(range(n), False)]
    a, b = loop["start"], loop["stop"]
    return [(range(a), False)] + [(range(a, b), True)] * loop["times"] \
        + [(range(b, n), False)]


def forward(cfg, W, tokens):
    """(logits [T, vocab], residual stream after each layer run) of one whole
    sequence."""
    eps = cfg["norm"]["eps"]
    W = {k: w.to(F64) for k, w in W.items()}
    x = start = W["embed"][torch.as_tensor(tokens).long()]
    stream = []
    for which, joined in passes(cfg):
        if joined:
            x = torch.cat([x, start], -1) @ W["loop.in"].T
        for i in which:
            x = layer(x, W, i, cfg["layers"][i], eps)
            stream.append(x)
    logits = rms_norm(x, W["final.norm"], eps) @ W["head"].T
    return logits, torch.stack(stream)
