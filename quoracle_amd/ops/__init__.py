"""quoracle_amd.ops — HIP/CDNA4 kernels (gfx950) with fail-loud loading.

On a GPU box the extension MUST be present: every op raises if the native
module failed to import, so a silent eager fallback can never masquerade as
the HIP path.  CPU-side tests use ops.reference (plain fp32 PyTorch
implementations of the same ops) as the numerics baseline.
"""

from __future__ import annotations

import importlib.util
import os
from typing import Dict

_HERE = os.path.dirname(os.path.abspath(__file__))

_loaded: Dict[str, object] = {}
_load_errors: Dict[str, str] = {}


def _load(name: str):
    if name in _loaded:
        return _loaded[name]
    path = os.path.join(_HERE, name + ".so")
    if not os.path.exists(path):
        _load_errors[name] = f"native extension not built: {path} missing " \
                             "(run quoracle_amd/ops/build.py)"
        return None
    try:
        spec = importlib.util.spec_from_file_location(name, path)
        mod = importlib.util.module_from_spec(spec)
        spec.loader.exec_module(mod)
    except Exception as exc:  # noqa: BLE001
        _load_errors[name] = f"native extension failed to load: {exc}"
        return None
    _loaded[name] = mod
    return mod


def _require(name: str):
    mod = _load(name)
    if mod is None:
        raise RuntimeError(
            f"quoracle_amd HIP extension unavailable: {_load_errors[name]}")
    return mod


def available() -> bool:
    return _load("_quoracle_ops") is not None


def ext():
    """The native module; raises loudly when missing (no silent fallback)."""
    return _require("_quoracle_ops")


def module(name: str):
    """A native module by its name; raises when missing."""
    return _require(name)


def hybrid_ext():
    """The kernels of recurrent and chunk-local mixers; raises when missing."""
    return _require("_quoracle_hybrid")


def latent_ext():
    """The kernels of latent attention and of mixtures of experts; raises
    when missing."""
    return _require("_quoracle_latent")


def stream_ext():
    """A module with the embedding and final-norm kernels that all hybrid
    models share: the one that is loaded, or any that is built."""
    for name in ("_quoracle_latent", "_quoracle_hybrid"):
        if name in _loaded:
            return _loaded[name]
    return _load("_quoracle_latent") or hybrid_ext()


# -- thin wrappers -----------------------------------------------------------

def rmsnorm_fused(y, x, residual, w, eps: float = 1e-5):
    ext().rmsnorm_fused(y, x, residual, w, eps)
    return y


def swiglu(out, gate_up):
    ext().swiglu(out, gate_up)
    return out


def rope_inplace(q, k, pos, theta: float = 500000.0):
    ext().rope_inplace(q, k, pos, theta)


def kv_append(kcache, vcache, k, v, slots):
    ext().kv_append(kcache, vcache, k, v, slots)


def paged_attn_decode(out, q, kcache, vcache, block_tables, ctx_lens,
                      scale: float):
    ext().paged_attn_decode(out, q, kcache, vcache, block_tables, ctx_lens,
                            scale)
    return out


def paged_attn_prefill(out, q, kcache, vcache, block_tables, tile_q0, tile_qn,
                       tile_seq, tile_pos0, scale: float):
    ext().paged_attn_prefill(out, q, kcache, vcache, block_tables, tile_q0,
                             tile_qn, tile_seq, tile_pos0, scale)
    return out


def cosine_sim_matrix(out, x):
    ext().cosine_sim_matrix(out, x)
    return out


def gather_rows(out, src, rows):
    ext().gather_rows(out, src, rows)
    return out


def paged_attn_decode_split(out, q, kcache, vcache, block_tables, ctx_lens,
                            scale, part_m, part_l, part_acc):
    ext().paged_attn_decode_split(out, q, kcache, vcache, block_tables,
                                  ctx_lens, scale, part_m, part_l, part_acc)
    return out


def paged_attn_prefill_mfma(out, q, kcache, vcache, block_tables, tile_q0,
                            tile_qn, tile_seq, tile_pos0, scale):
    ext().paged_attn_prefill_mfma(out, q, kcache, vcache, block_tables,
                                  tile_q0, tile_qn, tile_seq, tile_pos0,
                                  scale)
    return out


def paged_attn_prefill_mfma32(out, q, kcache, vcache, block_tables, tile_q0,
                              tile_qn, tile_seq, tile_pos0, scale):
    ext().paged_attn_prefill_mfma32(out, q, kcache, vcache, block_tables,
                                    tile_q0, tile_qn, tile_seq, tile_pos0,
                                    scale)
    return out
