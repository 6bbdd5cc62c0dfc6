"""Plain-PyTorch fp32 reference implementations of the HIP ops.

These are the numerics baselines the GPU tests compare the HIP kernels
against (tests/test_ops_gpu.py), and the compute path of the CPU reference
engine used by orchestrator tests.  Everything here is deliberately naive and
readable — correctness over speed.
"""

from __future__ import annotations

from typing import Optional, Tuple

import torch


def rmsnorm(x: torch.Tensor, w: torch.Tensor,
            residual: Optional[torch.Tensor] = None,
            eps: float = 1e-5) -> Tuple[torch.Tensor, Optional[torch.Tensor]]:
    """Returns (y, updated_residual)."""
    xf = x.float()
    if residual is not None:
        xf = xf + residual.float()
        residual = xf
    var = xf.pow(2).mean(dim=-1, keepdim=True)
    y = xf * torch.rsqrt(var + eps) * w.float()
    return y, residual


def swiglu(gate_up: torch.Tensor) -> torch.Tensor:
    inter = gate_up.shape[-1] // 2
    gate = gate_up[..., :inter].float()
    up = gate_up[..., inter:].float()
    return torch.nn.functional.silu(gate) * up


def rope(x: torch.Tensor, pos: torch.Tensor,
         theta: float = 500000.0) -> torch.Tensor:
    """Rotate-half RoPE. x: [T, H, D]; pos: [T]."""
    T, H, D = x.shape
    half = D // 2
    xf = x.float()
    freqs = theta ** (-2.0 * torch.arange(half, dtype=torch.float32,
                                          device=x.device) / D)
    angles = pos.float()[:, None] * freqs[None, :]        # [T, half]
    cos = angles.cos()[:, None, :]
    sin = angles.sin()[:, None, :]
    x0, x1 = xf[..., :half], xf[..., half:]
    return torch.cat([x0 * cos - x1 * sin, x0 * sin + x1 * cos], dim=-1)


def attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
              scale: float, causal_offset: Optional[int] = None) -> torch.Tensor:
    """q: [Tq, Hq, D]; k/v: [Tk, Hkv, D] (full context, oldest first).

    causal_offset: absolute position of q row 0; q row i attends to
    positions <= causal_offset + i.  None = attend to everything (decode
    with Tq=1 uses causal_offset = Tk-1 equivalently).
    """
    Tq, Hq, D = q.shape
    Tk, Hkv, _ = k.shape
    gq = Hq // Hkv
    qf = q.float()
    kf = k.float().repeat_interleave(gq, dim=1)   # [Tk, Hq, D]
    vf = v.float().repeat_interleave(gq, dim=1)
    scores = torch.einsum("qhd,khd->hqk", qf, kf) * scale
    if causal_offset is not None:
        kv_pos = torch.arange(Tk, device=q.device)[None, :]
        q_pos = causal_offset + torch.arange(Tq, device=q.device)[:, None]
        scores = scores.masked_fill((kv_pos > q_pos)[None], float("-inf"))
    probs = torch.softmax(scores, dim=-1)
    return torch.einsum("hqk,khd->qhd", probs, vf)


def cosine_sim_matrix(x: torch.Tensor) -> torch.Tensor:
    xf = x.float()
    norms = xf.norm(dim=-1, keepdim=True)
    safe = torch.where(norms > 0, norms, torch.ones_like(norms))
    xn = xf / safe
    sim = xn @ xn.T
    zero = (norms.squeeze(-1) == 0)
    sim[zero, :] = 0.0
    sim[:, zero] = 0.0
    return sim


# -- paged-KV reference implementations (same layouts as the HIP kernels) ----
# kcache/vcache: [NB, Hkv, BS, D]; block_tables: [B, MAXB] int32;
# slots: [T] int32 global slot = block*BS + offset.

def kv_append(kcache: torch.Tensor, vcache: torch.Tensor,
              k: torch.Tensor, v: torch.Tensor, slots: torch.Tensor) -> None:
    NB, Hkv, BS, D = kcache.shape
    for t in range(slots.shape[0]):
        s = int(slots[t])
        if s < 0:
            continue
        blk, off = s // BS, s % BS
        kcache[blk, :, off, :] = k[t]
        vcache[blk, :, off, :] = v[t]


def _gather_kv(cache: torch.Tensor, block_table: torch.Tensor,
               length: int) -> torch.Tensor:
    """[len, Hkv, D] rows 0..len-1 of one sequence from the paged cache."""
    NB, Hkv, BS, D = cache.shape
    toks = torch.arange(length, device=cache.device)
    blocks = block_table[toks // BS].long()
    offs = toks % BS
    return cache[blocks, :, offs, :]          # [len, Hkv, D]


def paged_attn_decode(out: torch.Tensor, q: torch.Tensor,
                      kcache: torch.Tensor, vcache: torch.Tensor,
                      block_tables: torch.Tensor, ctx_lens: torch.Tensor,
                      scale: float) -> torch.Tensor:
    B = q.shape[0]
    for b in range(B):
        length = int(ctx_lens[b])
        k = _gather_kv(kcache, block_tables[b], length)
        v = _gather_kv(vcache, block_tables[b], length)
        out[b] = attention(q[b:b + 1].float(), k, v, scale)[0].to(out.dtype)
    return out


def paged_attn_prefill(out: torch.Tensor, q: torch.Tensor,
                       kcache: torch.Tensor, vcache: torch.Tensor,
                       block_tables: torch.Tensor,
                       tile_q0: torch.Tensor, tile_qn: torch.Tensor,
                       tile_seq: torch.Tensor, tile_pos0: torch.Tensor,
                       scale: float) -> torch.Tensor:
    for t in range(tile_q0.shape[0]):
        q0, qn = int(tile_q0[t]), int(tile_qn[t])
        seq, pos0 = int(tile_seq[t]), int(tile_pos0[t])
        kv_len = pos0 + qn
        k = _gather_kv(kcache, block_tables[seq], kv_len)
        v = _gather_kv(vcache, block_tables[seq], kv_len)
        o = attention(q[q0:q0 + qn].float(), k, v, scale, causal_offset=pos0)
        out[q0:q0 + qn] = o.to(out.dtype)
    return out


def gather_rows(out: torch.Tensor, src: torch.Tensor,
                rows: torch.Tensor) -> torch.Tensor:
    out.copy_(src[rows.long()])
    return out


# -- hybrid models: recurrent mixers and chunk-local attention ---------------

def _rms(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x * torch.rsqrt(x.square().mean(-1, keepdim=True) + eps) * w.float()


def _act(x: torch.Tensor, act: int) -> torch.Tensor:
    """0 none, 1 silu, 2 sigmoid (the kernels' selectors)."""
    if act == 1:
        return torch.nn.functional.silu(x)
    return torch.sigmoid(x) if act == 2 else x


def embed_positions(x, h, embed, table, tokens, positions) -> None:
    v = embed[tokens.long()].float()
    if table is not None:
        v = v + table[positions.long()].float()
    x.copy_(v)
    h.copy_(v)


def post_norm(x, h, a, sa, b, sb, alpha, w, eps) -> None:
    y = alpha * x + sa * a.float()
    if b is not None:
        y = y + sb * b.float()
    x.copy_(_rms(y, w, eps))
    h.copy_(x)


def norm_rows(out, x, rows, w, eps) -> None:
    out.copy_(_rms(x[rows], w, eps))


def gated_norm(out, o, proj, g_off, w, groups, act, eps) -> None:
    T, n = o.shape[0], w.shape[0]
    y = _rms(o.float().view(T, groups, n), w, eps).view(T, groups * n)
    gate = proj[:, g_off:g_off + groups * n].float()
    out.copy_((y * _act(gate, act)).view_as(out))


def rope_interleaved(x: torch.Tensor, pos: torch.Tensor, freq: torch.Tensor,
                     mag: float) -> torch.Tensor:
    """Rotate the pairs (2i, 2i+1), i < len(freq), of x [T, H, D]."""
    n = freq.shape[0]
    ang = pos.double()[:, None] * freq.double()[None, :]
    cos = (ang.cos().float() * mag)[:, None, :]
    sin = (ang.sin().float() * mag)[:, None, :]
    pairs = x[..., :2 * n].unflatten(-1, (n, 2))
    u, v = pairs[..., 0], pairs[..., 1]
    turned = torch.stack([u * cos - v * sin, v * cos + u * sin], dim=-1)
    return torch.cat([turned.flatten(-2), x[..., 2 * n:]], dim=-1)


def qk_norm_rope_store(q_out, kcache, vcache, proj, q_off, k_off, qw, kw,
                       positions, slots, freq, mag, eps) -> None:
    T, H, D = q_out.shape
    G = kcache.shape[1]
    raw = proj[:, k_off:k_off + G * D].float()
    q = _rms(proj[:, q_off:q_off + H * D].float(), qw, eps).view(T, H, D)
    k = _rms(raw, kw, eps).view(T, G, D)
    q_out.copy_(rope_interleaved(q, positions, freq, mag))
    k = rope_interleaved(k, positions, freq, mag).to(kcache.dtype)
    kv_append(kcache, vcache, k, raw.view(T, G, D).to(vcache.dtype), slots)


def local_attention(out, q, kcache, vcache, block_tables, row_seq, positions,
                    scale, chunk, sink) -> None:
    gq = q.shape[1] // kcache.shape[1]
    for seq in row_seq.unique().tolist():
        rows = (row_seq == seq).nonzero(as_tuple=True)[0]
        pos = positions[rows].long()
        length = int(pos.max()) + 1
        k = _gather_kv(kcache, block_tables[seq], length).float()
        v = _gather_kv(vcache, block_tables[seq], length).float()
        k, v = k.repeat_interleave(gq, 1), v.repeat_interleave(gq, 1)
        s = torch.einsum("qhd,khd->hqk", q[rows].float(), k) * scale
        key = torch.arange(length)
        ok = key[None, :] <= pos[:, None]
        if chunk > 0:
            ok &= (key // chunk)[None, :] == (pos // chunk)[:, None]
        s = s.masked_fill(~ok[None], float("-inf"))
        if sink:
            s = torch.cat([s, torch.zeros_like(s[..., :1])], dim=-1)
        p = torch.softmax(s, dim=-1)[..., :length]
        out[rows] = torch.einsum("hqk,khd->qhd", p, v).to(out.dtype)


def log_decay(out, proj, a_off, a2, bias, tau) -> None:
    a = proj[:, a_off:a_off + a2.shape[1]].float()
    z = a @ a2.float().T + bias
    out.copy_(torch.nn.functional.logsigmoid(z) / tau)


def linear_attention(o, proj, q_off, k_off, v_off, act, qscale, decay,
                     channel, state, slots, row_seq, positions) -> None:
    H, V, D = state.shape[1:]
    T = proj.shape[0]
    q = _act(proj[:, q_off:q_off + H * D].float(), act).view(T, H, D)
    k = _act(proj[:, k_off:k_off + H * D].float(), act).view(T, H, D)
    v = _act(proj[:, v_off:v_off + H * V].float(), act).view(T, H, V)
    a = decay.exp().view(T, H, D) if channel \
        else decay[None, :, None].expand(T, H, D)
    y = torch.empty(T, H, V)
    for t in range(T):          # rows of a sequence come in order
        slot = int(slots[int(row_seq[t])])
        if int(positions[t]) == 0:
            state[slot].zero_()
        S = state[slot]
        S.mul_(a[t][:, None, :]).add_(v[t][:, :, None] * k[t][:, None, :])
        y[t] = (S @ q[t][:, :, None]).squeeze(-1) * qscale
    o.copy_(y.view_as(o))


# -- latent attention, mixtures of experts, norms around a sublayer ----------

def pre_norm(x, h, y, w, eps) -> None:
    if y is not None:
        x.copy_(y)
    h.copy_(_rms(x, w, eps))


def sandwich_norm(x, h, joined, w_next, y, bias, y2, gate, w, eps) -> None:
    s = y.float()
    if s.dim() == 3:
        s = s.sum(1)
    if bias is not None:
        s = s + bias
    if y2 is not None:
        s = s + gate[:, None] * y2.float()
    x += _rms(s, w, eps)
    if w_next is not None:
        h.copy_(_rms(x, w_next, eps))
    if joined is not None:
        joined[:, :x.shape[1]] = x.to(joined.dtype)


def latent_store(cq, pool, proj, kv_off, rank_p, wq, wkv, positions, slots,
                 freq, eps) -> None:
    bs = pool.shape[1]
    rank, n = wkv.shape[0], 2 * freq.shape[0]
    cq.copy_(_rms(proj[:, :wq.shape[0]].float(), wq, eps))
    c = _rms(proj[:, kv_off:kv_off + rank].float(), wkv, eps)
    k = rope_interleaved(
        proj[:, None, kv_off + rank:kv_off + rank + n].float(), positions,
        freq, 1.0)[:, 0]
    row = torch.zeros(c.shape[0], pool.shape[2])
    row[:, :rank] = c
    row[:, rank_p:rank_p + n] = k
    at = slots.long()
    pool[at // bs, at % bs] = row.to(pool.dtype)


def rotate_heads(q, off, positions, freq) -> None:
    n = 2 * freq.shape[0]
    part = q[..., off:off + n].float()
    q[..., off:off + n] = rope_interleaved(part, positions, freq,
                                           1.0).to(q.dtype)


def latent_attention(out, q, pool, w_kv, sink, scale, block_tables, row_seq,
                     positions) -> None:
    T, H, V = out.shape
    rot = pool.shape[2] - w_kv.shape[1]
    dim = q.shape[2] - rot
    rank = w_kv.shape[1]
    w = w_kv.float()
    for seq in row_seq.unique().tolist():
        rows = (row_seq == seq).nonzero(as_tuple=True)[0]
        pos = positions[rows].long()
        length = int(pos.max()) + 1
        blocks = block_tables[seq, :-(-length // pool.shape[1])].long()
        ctx = pool[blocks].flatten(0, 1)[:length].float()
        kv = ctx[:, :rank] @ w.T
        k = torch.cat([kv[:, :H * dim].view(length, H, dim),
                       ctx[:, None, rank:].expand(length, H, rot)], -1)
        v = kv[:, H * dim:].view(length, H, V)
        s = torch.einsum("qhd,khd->hqk", q[rows].float(), k) * scale
        s = s.masked_fill(torch.arange(length)[None, None, :]
                          > pos[None, :, None], float("-inf"))
        if sink is not None:
            s = torch.cat([s, sink[:, None, None].expand(H, len(rows), 1)],
                          dim=-1)
        p = torch.softmax(s, dim=-1)[..., :length]
        out[rows] = torch.einsum("hqk,khd->qhd", p, v).to(out.dtype)


def bias_gelu(up, bias) -> None:
    v = up.float() if bias is None else up.float() + bias
    up.copy_(torch.nn.functional.gelu(v))


def moe_route(ids, weights, gate, h, router, experts) -> None:
    s = torch.sigmoid(h.float() @ router.float().T)
    w, i = s[:, :experts].topk(ids.shape[1], dim=-1)
    ids.copy_(i)
    weights.copy_(w)
    if gate is not None:
        gate.copy_(s[:, experts])


def moe_experts(y, h, ids, weights, up, down) -> None:
    for e in ids.unique().tolist():
        t, k = (ids == e).nonzero(as_tuple=True)
        z = (h[t].float() @ up[e].float().T) * weights[t, k, None]
        a = torch.nn.functional.gelu(z)
        y[t, k] = (a @ down[e].float().T).to(y.dtype)
