"""Device dispatch of latent attention, of mixtures of experts and of the
norms around a sublayer.

GPU tensors go to the HIP extension, which must be there; CPU tensors go to
the plain implementations in ops/reference.py (same rule as ops/dispatch.py).
"""

from __future__ import annotations

from typing import Optional

import torch
import torch.nn.functional as F

from . import latent_ext
from . import reference as ref


def tiles_ok(spec, dtype: torch.dtype) -> bool:
    """The matrix-core kernels in the latent space take these sizes."""
    return dtype == torch.bfloat16 and spec.rank_p <= 512 \
        and spec.rot_p <= 64


def expandable(spec) -> bool:
    """The prefill tile over expanded keys and values takes these sizes."""
    return spec.dim_p + spec.rot_p <= 256 and spec.vdim_p <= 256


def linear_f32(a, w) -> torch.Tensor:
    """a w^T with a float32 result."""
    if a.is_cuda and a.dtype != torch.float32:
        return torch.mm(a, w.t(), out_dtype=torch.float32)
    return F.linear(a, w).float()


def pre_norm(x, h, y: Optional[torch.Tensor], w, eps: float) -> None:
    """x = y if given; h = rms(x) * w."""
    if x.is_cuda:
        latent_ext().pre_norm(x, h, y, w, eps)
        return
    ref.pre_norm(x, h, y, w, eps)


def sandwich_norm(x, h, joined: Optional[torch.Tensor],
                  w_next: Optional[torch.Tensor], y,
                  bias: Optional[torch.Tensor], y2: Optional[torch.Tensor],
                  gate: Optional[torch.Tensor], w, eps: float) -> None:
    """x += rms(sum of y [T, (K,) n] + bias + gate * y2) * w; then
    h = rms(x) * w_next and joined[:, :n] = x where they are given."""
    if x.is_cuda:
        latent_ext().sandwich_norm(x, h, joined, w_next, y, bias, y2, gate, w,
                                   eps)
        return
    ref.sandwich_norm(x, h, joined, w_next, y, bias, y2, gate, w, eps)


def latent_store(cq, pool, proj, kv_off: int, rank_p: int, wq, wkv, positions,
                 slots, freq, eps: float) -> None:
    """Rows of the fused projection -> normed query latent, and the normed
    latent and rotated key part in the paged pool."""
    if proj.is_cuda:
        latent_ext().latent_store(cq, pool, proj, kv_off, rank_p, wq, wkv,
                                  positions, slots, freq, eps)
        return
    ref.latent_store(cq, pool, proj, kv_off, rank_p, wq, wkv, positions,
                     slots, freq, eps)


def rotate_heads(q, off: int, positions, freq) -> None:
    """Rotate the interleaved pairs of q[..., off:off + 2 len(freq)] in
    place."""
    if q.is_cuda:
        latent_ext().rotate_heads(q, off, positions, freq)
        return
    ref.rotate_heads(q, off, positions, freq)


def latent_attention(out, q, pool, w_kv, w_uk_t, sink, scale: float,
                     batch) -> None:
    """Attention of every row of a ForwardBatch over the paged latents: q
    [T, H, dim + rot], pool [blocks, BS, rank + rot], w_kv the keys' and then
    the values' rows of every head, w_uk_t [H, rank, dim] the keys' part
    transposed."""
    if not q.is_cuda:
        ref.latent_attention(out, q, pool, w_kv, sink, scale,
                             batch.block_tables, batch.row_seq,
                             batch.positions)
        return
    latent_ext().latent_attention(out, q, pool, w_kv, w_uk_t, sink, scale,
                                  batch.hybrid_tensors(),
                                  batch.hybrid_numbers())


def bias_gelu(up, bias: Optional[torch.Tensor]) -> None:
    """up = gelu(up + bias) in place, the exact form."""
    if up.is_cuda:
        latent_ext().bias_gelu(up, bias)
        return
    ref.bias_gelu(up, bias)


def moe_route(ids, weights, gate: Optional[torch.Tensor], h, router,
              experts: int) -> None:
    """The chosen experts of each row and their sigmoid scores; `gate`: the
    sigmoid of the router row behind the experts'."""
    if h.is_cuda:
        latent_ext().moe_route(ids, weights, gate, h, router, experts)
        return
    ref.moe_route(ids, weights, gate, h, router, experts)


def moe_experts(y, h, ids, weights, up, down) -> None:
    """y[t, k] = down_e gelu(up_e (weights[t, k] * h[t])), e = ids[t, k]."""
    if h.is_cuda:
        latent_ext().moe_experts(y, h, ids, weights, up, down)
        return
    ref.moe_experts(y, h, ids, weights, up, down)
