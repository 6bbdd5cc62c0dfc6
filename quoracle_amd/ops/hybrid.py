"""Device dispatch of the hybrid-model ops.

GPU tensors go to the HIP extension, which must be there; CPU tensors go to
the plain implementations in ops/reference.py so that the engine is testable
without a GPU (same rule as ops/dispatch.py).

`proj` arguments are the rows of a layer's fused input projection; the
`*_off` arguments are element offsets of one part inside such a row.
"""

from __future__ import annotations

from typing import Optional

import torch

from . import hybrid_ext, stream_ext
from . import reference as ref

LIN_CHUNK = 64          # tokens per linear-attention chunk (csrc LIN_CHUNK)
ATTN_TILE = 128         # query rows per prefill attention tile

ACT_NONE, ACT_SILU, ACT_SIGMOID = 0, 1, 2


def embed_positions(x, h, embed, table: Optional[torch.Tensor], tokens,
                    positions) -> None:
    """x = embed[tokens] (+ table[positions]) in float32; h = x in h's type."""
    if x.is_cuda:
        stream_ext().embed_positions(x, h, embed, table, tokens, positions)
        return
    ref.embed_positions(x, h, embed, table, tokens, positions)


def post_norm(x, h, a, sa: float, b: Optional[torch.Tensor], sb: float,
              alpha: float, w, eps: float) -> None:
    """x <- rms(alpha*x + sa*a (+ sb*b)) * w in place; h = x in h's type."""
    if x.is_cuda:
        hybrid_ext().post_norm(x, h, a, sa, b, sb, alpha, w, eps)
        return
    ref.post_norm(x, h, a, sa, b, sb, alpha, w, eps)


def norm_rows(out, x, rows, w, eps: float) -> None:
    """out[r] = rms(x[rows[r]]) * w."""
    if x.is_cuda:
        stream_ext().norm_rows(out, x, rows, w, eps)
        return
    ref.norm_rows(out, x, rows, w, eps)


def glu(out, gate_up) -> None:
    if out.is_cuda:
        hybrid_ext().glu(out, gate_up)
        return
    out.copy_(ref.swiglu(gate_up).to(out.dtype))


def gated_norm(out, o, proj, g_off: int, w, groups: int, act: int,
               eps: float) -> None:
    """Norm each of `groups` groups of o, times w, times act(gate)."""
    if out.is_cuda:
        hybrid_ext().gated_norm(out, o, proj, g_off, w, groups, act, eps)
        return
    ref.gated_norm(out, o, proj, g_off, w, groups, act, eps)


def qk_norm_rope_store(q_out, kcache, vcache, proj, q_off: int, k_off: int,
                       qw, kw, positions, slots, freq, mag: float,
                       eps: float) -> None:
    """Norm queries and keys over their whole projection, rotate interleaved
    pairs, store rotated keys and raw keys (the values) in the paged cache."""
    if q_out.is_cuda:
        hybrid_ext().qk_norm_rope_store(q_out, kcache, vcache, proj, q_off,
                                        k_off, qw, kw, positions, slots, freq,
                                        mag, eps)
        return
    ref.qk_norm_rope_store(q_out, kcache, vcache, proj, q_off, k_off, qw, kw,
                           positions, slots, freq, mag, eps)


def local_attention(out, q, kcache, vcache, batch, scale: float, chunk: int,
                    sink: bool) -> None:
    """Attention of every row of a ForwardBatch over the paged cache, confined
    to position chunks of `chunk` tokens (0: unconfined); `sink` adds one to
    the softmax denominator."""
    if not q.is_cuda:
        ref.local_attention(out, q, kcache, vcache, batch.block_tables,
                            batch.row_seq, batch.positions, scale, chunk,
                            sink)
        return
    e = hybrid_ext()
    if not e.attn_tiles_ok(q) or q.shape[1] // kcache.shape[1] > 16:
        e.local_attn_rows(out, q, kcache, vcache, batch.block_tables,
                          batch.row_seq, batch.positions, scale, chunk, sink)
        return
    if batch.n_decode:
        e.local_attn_decode(out, q, kcache, vcache, batch.block_tables,
                            batch.ctx_lens, scale, chunk, sink, batch.max_ctx)
    if batch.total_tokens > batch.n_decode:
        e.local_attn_prefill(out, q, kcache, vcache, batch.block_tables,
                             batch.tile32_q0, batch.tile32_qn,
                             batch.tile32_seq, batch.tile32_pos0, scale,
                             chunk, sink, batch.max_kv)


def log_decay(out, proj, a_off: int, a2, bias, tau: float, batch,
              state) -> None:
    """log(sigmoid(A2 a + b)) / tau per row and key channel; on the GPU summed
    along each prefill chunk where the chunked form will read it."""
    if not out.is_cuda:
        ref.log_decay(out, proj, a_off, a2, bias, tau)
        return
    e = hybrid_ext()
    if not e.linear_tiles_ok(proj, state):
        e.log_decay(out, proj, a_off, a2, bias, tau, 0, proj.shape[0], None,
                    None)
        return
    e.log_decay(out, proj, a_off, a2, bias, tau, 0, batch.n_decode, None,
                None)
    if batch.total_tokens > batch.n_decode:
        e.log_decay(out, proj, a_off, a2, bias, tau, 0, 0, batch.chunk_row0,
                    batch.chunk_len)


def linear_attention(o, proj, q_off: int, k_off: int, v_off: int, act: int,
                     qscale: float, decay, powers, channel: bool, state,
                     batch) -> None:
    """S_t = diag(a_t) S_(t-1) + k_t v_t^T, o_t = qscale * S_t^T q_t for every
    sequence of a ForwardBatch, from and into the state pool
    [slots, H, V, D].  `decay`: one constant per head [H], or with `channel`
    what log_decay gave; `powers`: of each head's constant, [H, LIN_CHUNK+1].
    """
    n = batch.n_decode
    slots = batch.state_slots
    if not o.is_cuda:
        ref.linear_attention(o, proj, q_off, k_off, v_off, act, qscale, decay,
                             channel, state, slots, batch.row_seq,
                             batch.positions)
        return
    e = hybrid_ext()
    if n:
        e.linear_recurrent(o, proj, q_off, k_off, v_off, act, qscale, decay,
                           channel, state, None, None, slots[:n],
                           batch.positions)
    if batch.total_tokens > n:
        if e.linear_tiles_ok(proj, state):
            e.linear_chunked(o, proj, q_off, k_off, v_off, act, qscale,
                             decay if channel else powers, channel, state,
                             batch.chunk_row0, batch.chunk_len,
                             batch.seg_row0, batch.seg_chunk0, slots[n:],
                             batch.positions)
        else:
            e.linear_recurrent(o, proj, q_off, k_off, v_off, act, qscale,
                               decay, channel, state, batch.seg_row0,
                               batch.seg_len, slots[n:], batch.positions)
