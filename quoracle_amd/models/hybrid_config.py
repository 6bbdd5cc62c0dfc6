"""Configurations of hybrid models: layers that mix tokens with a recurrent
state, with chunk-local attention, or with both side by side.

The specs describe mechanisms and carry every constant as a parameter; an
architecture (Koridra) is a reader of its config.json plus an order of specs.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple


@dataclass(frozen=True)
class RotarySpec:
    """Interleaved rotary positions on the first `dims` dimensions, with YaRN
    frequency scaling when `factor` is set."""
    dims: int
    base: float
    factor: Optional[float] = None
    original: float = 0.0
    fast: float = 32.0
    slow: float = 1.0

    def frequencies(self) -> Tuple[Tuple[float, ...], float]:
        """(angle per position of each pair, factor on cos and sin)."""
        n = self.dims // 2
        plain = [self.base ** (-2.0 * i / self.dims) for i in range(n)]
        if self.factor is None:
            return tuple(plain), 1.0

        def turns_at(turns: float) -> float:
            # dimension index whose wave makes `turns` turns in `original`
            return (self.dims * math.log(self.original
                                         / (2.0 * math.pi * turns))
                    / (2.0 * math.log(self.base)))

        lo = max(math.floor(turns_at(self.fast)), 0)
        hi = min(math.ceil(turns_at(self.slow)), self.dims - 1)
        span = max(hi - lo, 0.001)
        out = []
        for i, f in enumerate(plain):
            ramp = min(1.0, max(0.0, (i - lo) / span))
            out.append(f * (ramp / self.factor + 1.0 - ramp))
        return tuple(out), 0.1 * math.log(self.factor) + 1.0


@dataclass(frozen=True)
class LocalAttentionSpec:
    """GQA attention inside position chunks of `chunk` tokens (0: unconfined).
    The values are the projected keys; queries and keys are RMS-normed over
    their whole projection; `sink` adds one to the softmax denominator."""
    heads: int
    kv_heads: int
    dim: int
    scale: float
    chunk: int
    rotary: Optional[RotarySpec]
    sink: bool = True


@dataclass(frozen=True)
class LinearAttentionSpec:
    """Linear attention with a decaying [dim, vdim] state per head.

    `decay`: one constant per head; None: a decay per key channel and token,
    sigmoid(low-rank projection) ** (1/tau), of rank `rank` (None: whatever
    the checkpoint holds).  `act` is applied to q, k and v; the output is
    RMS-normed over each head (`head_norm`) or over all heads together and
    multiplied by `gate_act` of a gate."""
    heads: int
    dim: int
    vdim: int
    act: str
    gate_act: str
    head_norm: bool
    qscale: float
    decay: Optional[Tuple[float, ...]] = None
    tau: float = 1.0
    rank: Optional[int] = None

    @property
    def state_elements(self) -> int:
        return self.heads * self.dim * self.vdim


def lightning(heads: int, dim: int, vdim: int,
              decay: Tuple[float, ...]) -> LinearAttentionSpec:
    if len(decay) != heads:
        raise ValueError(f"{heads} heads but {len(decay)} decays")
    return LinearAttentionSpec(heads, dim, vdim, act="silu",
                               gate_act="sigmoid", head_norm=False,
                               qscale=1.0, decay=tuple(decay))


def gated_linear(heads: int, dim: int, vdim: int, tau: float,
                 rank: Optional[int] = None) -> LinearAttentionSpec:
    return LinearAttentionSpec(heads, dim, vdim, act="none", gate_act="silu",
                               head_norm=True, qscale=dim ** -0.5, tau=tau,
                               rank=rank)


@dataclass(frozen=True)
class HybridLayerSpec:
    """One layer; attn and linear side by side when both are given."""
    attn: Optional[LocalAttentionSpec] = None
    linear: Optional[LinearAttentionSpec] = None
    attn_scale: float = 1.0
    linear_scale: float = 1.0
    ff: Optional[int] = None
    kind: str = ""


@dataclass(frozen=True)
class KoridraConfig:
    """Koridra: lightning layers and layers of attention beside gated linear
    attention, learned positions, norm after the sum."""
    name: str
    vocab_size: int
    hidden: int
    layers: Tuple[HybridLayerSpec, ...]
    alpha: float
    rmsnorm_eps: float
    max_context: int
    max_output: int = 4096
    path: Optional[str] = None          # checkpoint folder; None: random init

    architecture = "Koridra"
    native_module = "_quoracle_hybrid"
    is_hybrid = True
    is_moe = False

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @property
    def needs_state(self) -> bool:
        return any(s.linear is not None for s in self.layers)

    def kv_bytes_per_token(self, element: int = 2) -> int:
        return 2 * element * sum(s.attn.kv_heads * s.attn.dim
                                 for s in self.layers if s.attn)

    def state_bytes_per_sequence(self) -> int:
        return 4 * sum(s.linear.state_elements
                       for s in self.layers if s.linear)

    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        """Checkpoint tensor names and shapes ([out, in] matrices); a rank of
        0 is one that only the checkpoint knows."""
        w = self.hidden
        t: Dict[str, Tuple[int, ...]] = {
            "embed": (self.vocab_size, w), "pos": (self.max_context, w)}
        for i, s in enumerate(self.layers):
            p = f"l{i}."
            t[p + "norm1"] = (w,)
            a, lin = s.attn, s.linear
            ap, lp = ((p + "mix.left.", p + "mix.right.") if a
                      else ("", p + "mix."))
            if a:
                nq, nk = a.heads * a.dim, a.kv_heads * a.dim
                t.update({ap + "q": (nq, w), ap + "k": (nk, w),
                          ap + "q.norm": (nq,), ap + "k.norm": (nk,),
                          ap + "o": (w, nq)})
            if lin:
                nk, nv = lin.heads * lin.dim, lin.heads * lin.vdim
                t.update({lp + "q": (nk, w), lp + "k": (nk, w),
                          lp + "v": (nv, w), lp + "g": (nv, w),
                          lp + "o": (w, nv),
                          lp + "norm": (lin.vdim if lin.head_norm else nv,)})
                if lin.decay is None:
                    r = lin.rank or 0
                    t.update({lp + "a1": (r, w), lp + "a2": (nk, r),
                              lp + "a2.b": (nk,)})
            if s.ff is not None:
                t.update({p + "mlp.gate": (s.ff, w), p + "mlp.up": (s.ff, w),
                          p + "mlp.down": (w, s.ff), p + "norm2": (w,)})
        t["final.norm"] = (w,)
        t["head"] = (self.vocab_size, w)
        return t

    def param_count(self) -> int:
        return sum(math.prod(s) for s in self.tensor_shapes().values())

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], name: str = "koridra",
                  path: Optional[str] = None) -> "KoridraConfig":
        context = int(raw["max_positions"])
        return cls(
            name=name, vocab_size=int(raw["vocab"]),
            hidden=int(raw["width"]),
            layers=tuple(_koridra_layer(e) for e in raw["layers"]),
            alpha=float(raw["postln_alpha"]),
            rmsnorm_eps=float(raw["norm"]["eps"]),
            max_context=context, max_output=min(4096, context), path=path)


def _rotary(raw: Optional[Dict[str, Any]]) -> Optional[RotarySpec]:
    if not raw:
        return None
    sc = raw.get("scaling") or {}
    return RotarySpec(
        dims=int(raw["dims"]), base=float(raw["base"]),
        factor=float(sc["factor"]) if sc else None,
        original=float(sc.get("original", 0.0)),
        fast=float(sc.get("fast", 32.0)), slow=float(sc.get("slow", 1.0)))


def _koridra_layer(raw: Dict[str, Any]) -> HybridLayerSpec:
    kind, m, mlp = raw["type"], raw["mixer"], raw.get("mlp")
    ff = None
    if mlp is not None:
        if mlp["kind"] != "dense":
            raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
        ff = int(mlp["ff"])
    if kind == "lightning":
        return HybridLayerSpec(
            linear=lightning(int(m["heads"]), int(m["dim"]), int(m["vdim"]),
                             tuple(float(d) for d in m["decay"])),
            ff=ff, kind=kind)
    if kind == "parallel":
        left, right = m["left"], m["right"]
        dim, heads, kv = (int(left[k]) for k in ("dim", "heads", "kv_heads"))
        if int(left.get("vdim", dim)) != dim:
            raise ValueError("values are the projected keys: vdim must be dim")
        if heads % kv:
            raise ValueError("heads must be a multiple of kv_heads")
        mask = left.get("mask") or {}
        return HybridLayerSpec(
            attn=LocalAttentionSpec(
                heads=heads, kv_heads=kv, dim=dim,
                scale=float(left["scale"]), chunk=int(mask.get("size", 0)),
                rotary=_rotary(left.get("rot"))),
            linear=gated_linear(int(right["heads"]), int(right["dim"]),
                                int(right["vdim"]), float(right["tau"])),
            attn_scale=float(m["left_scale"]),
            linear_scale=float(m["right_scale"]), ff=ff, kind=kind)
    raise ValueError(f"unknown mixer {kind!r}")


def koridra_preset(name: str, *, vocab: int, hidden: int, n_layers: int,
                   ff: int, heads: int, kv_heads: int, dim: int, chunk: int,
                   lin_heads: int, lin_dim: int, lin_vdim: int,
                   max_context: int, every: int = 4, max_output: int = 4096,
                   base: float = 500000.0, rank: int = 16) -> KoridraConfig:
    """Random-weight Koridra: one parallel layer in `every`, slowest decays
    spread geometrically over the heads."""
    decay = tuple(math.exp(-2.0 ** (-8.0 * (h + 1) / lin_heads))
                  for h in range(lin_heads))
    layers = []
    for i in range(n_layers):
        if i % every == every - 1:
            layers.append(HybridLayerSpec(
                attn=LocalAttentionSpec(
                    heads, kv_heads, dim, scale=dim ** -0.5, chunk=chunk,
                    rotary=RotarySpec(dim, base, factor=4.0,
                                      original=max_context / 4)),
                linear=gated_linear(lin_heads, lin_dim, lin_vdim, tau=16.0,
                                    rank=rank),
                attn_scale=0.7, linear_scale=0.7, ff=ff, kind="parallel"))
        else:
            layers.append(HybridLayerSpec(
                linear=lightning(lin_heads, lin_dim, lin_vdim, decay), ff=ff,
                kind="lightning"))
    return KoridraConfig(name=name, vocab_size=vocab, hidden=hidden,
                         layers=tuple(layers),
                         alpha=(2.0 * n_layers) ** 0.25, rmsnorm_eps=1e-5,
                         max_context=max_context, max_output=max_output)
