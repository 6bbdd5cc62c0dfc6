"""Plain, slow Koridra in float64: one function per mechanism.

Token by token and pair by pair, straight from the equations, over a dict of
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


def silu(z):
    return z * torch.sigmoid(z)


def rotary_frequencies(rot):
    """(frequency per pair, factor on cos and sin), YaRN when rot.scaling."""
    dims, base = rot["dims"], rot["base"]
    freq = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return freq, 1.0

    def dim_of(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) \
            / (2 * math.log(base))

    lo = max(math.floor(dim_of(sc["fast"])), 0)
    hi = min(math.ceil(dim_of(sc["slow"])), dims - 1)
    out = []
    for i, f in enumerate(freq):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / sc["factor"] * ramp + f * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1


def rotate_interleaved(x, position, rot):
    """Rotate the pairs (2i, 2i+1) of one head vector; the rest passes."""
    freq, mag = rotary_frequencies(rot)
    y = x.clone()
    for i, f in enumerate(freq):
        c = math.cos(position * f) * mag
        s = math.sin(position * f) * mag
        u, v = x[2 * i], x[2 * i + 1]
        y[2 * i] = u * c - v * s
        y[2 * i + 1] = v * c + u * s
    return y


def sees(i, j, chunk):
    """Causal and inside the same chunk counted from position 0."""
    return j <= i and (not chunk or i // chunk == j // chunk)


def sink_attention(q, k, v, scale, chunk, positions=None):
    """q [Tq, H, D] at `positions` (default: all of 0..T-1) over k/v
    [T, G, *]; the softmax denominator has one added to it."""
    H, G = q.shape[1], k.shape[1]
    positions = range(k.shape[0]) if positions is None else positions
    out = torch.zeros(q.shape[0], H, v.shape[2], dtype=q.dtype)
    for r, i in enumerate(positions):
        js = [j for j in range(k.shape[0]) if sees(i, j, chunk)]
        for h in range(H):
            g = h // (H // G)
            s = (k[js, g] @ q[r, h]) * scale
            top = max(float(s.max()), 0.0)
            e = torch.exp(s - top)
            p = e / (math.exp(-top) + e.sum())
            out[r, h] = p @ v[js, g]
    return out


def decayed_recurrence(q, k, v, decay, state=None):
    """S_t = diag(decay_t) S_(t-1) + k_t v_t^T, o_t = S_t^T q_t per head.
    q, k [T, H, D], v [T, H, V]; decay broadcasts to [T, H, D].  Returns
    (o [T, H, V], state [H, D, V])."""
    T, H, D = q.shape
    V = v.shape[2]
    decay = decay.expand(T, H, D)
    S = torch.zeros(H, D, V, dtype=q.dtype) if state is None else state.clone()
    o = torch.zeros(T, H, V, dtype=q.dtype)
    for t in range(T):
        for h in range(H):
            S[h] = decay[t, h][:, None] * S[h] \
                + k[t, h][:, None] * v[t, h][None, :]
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def lightning_mixer(h, W, p, m, eps):
    """Decay fixed per head; the joined heads are normed together."""
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = silu(h @ W[p + "q"].T).view(T, H, D)
    k = silu(h @ W[p + "k"].T).view(T, H, D)
    v = silu(h @ W[p + "v"].T).view(T, H, V)
    decay = torch.tensor(m["decay"], dtype=h.dtype)[None, :, None]
    o, _ = decayed_recurrence(q, k, v, decay)
    o = rms_norm(o.reshape(T, H * V), W[p + "norm"], eps)
    return (o * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def gla_decay(h, W, p, tau):
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "a2.b"]
    return torch.sigmoid(z) ** (1.0 / tau)


def gla_mixer(h, W, p, m, eps):
    """Decay per key channel and token; each head is normed by itself."""
    T = h.shape[0]
    H, D, V = m["heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, D)
    v = (h @ W[p + "v"].T).view(T, H, V)
    decay = gla_decay(h, W, p, m["tau"]).view(T, H, D)
    o, _ = decayed_recurrence(q, k, v, decay)
    o = rms_norm(o, W[p + "norm"], eps).reshape(T, H * V)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def attention_mixer(h, W, p, m, eps):
    """The values are the projected keys, before norm and rotation."""
    T = h.shape[0]
    H, G, D = m["heads"], m["kv_heads"], m["dim"]
    raw = h @ W[p + "k"].T
    q = rms_norm(h @ W[p + "q"].T, W[p + "q.norm"], eps).view(T, H, D)
    k = rms_norm(raw, W[p + "k.norm"], eps).view(T, G, D)
    v = raw.view(T, G, D)
    q = torch.stack([torch.stack([rotate_interleaved(q[t, a], t, m["rot"])
                                  for a in range(H)]) for t in range(T)])
    k = torch.stack([torch.stack([rotate_interleaved(k[t, a], t, m["rot"])
                                  for a in range(G)]) for t in range(T)])
    o = sink_attention(q, k, v, m["scale"], m["mask"]["size"])
    return o.reshape(T, H * D) @ W[p + "o"].T


def parallel_mixer(h, W, p, m, eps):
    return (m["left_scale"] * attention_mixer(h, W, p + "left.", m["left"], eps)
            + m["right_scale"] * gla_mixer(h, W, p + "right.", m["right"], eps))


MIXERS = {"lightning": lightning_mixer, "parallel": parallel_mixer}


def dense_ff(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def forward(cfg, W, tokens):
    """(logits [T, vocab], residual stream after each layer [L, T, width])
    of one whole sequence."""
    eps, alpha = cfg["norm"]["eps"], cfg["postln_alpha"]
    W = {k: w.to(F64) for k, w in W.items()}
    x = W["embed"][torch.as_tensor(tokens).long()] + W["pos"][:len(tokens)]
    stream = []
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        mixed = MIXERS[spec["type"]](x, W, p + "mix.", spec["mixer"], eps)
        x = rms_norm(alpha * x + mixed, W[p + "norm1"], eps)
        if spec["mlp"] is not None:
            x = rms_norm(alpha * x + dense_ff(x, W, p + "mlp."),
                         W[p + "norm2"], eps)
        stream.append(x)
    logits = rms_norm(x, W["final.norm"], eps) @ W["head"].T
    return logits, torch.stack(stream)
