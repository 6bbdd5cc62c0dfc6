"""Configurations of hybrid models: layers that mix tokens with a recurrent
state, with chunk-local attention, with both side by side, or with attention
over cached latents.

The specs describe mechanisms and carry every constant as a parameter; an
architecture (Koridra, Kotutar) is a reader of its config.json plus an order
of specs.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple, Union


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


def _pad8(n: int) -> int:
    return n + -n % 8


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Causal attention whose keys and values are made from one cached latent
    of `kv_rank` values and one rotated key part of `rot_dim` values per
    token, both shared by all heads.  Queries pass through a normed latent of
    `q_rank` values and have `dim` plain and `rot_dim` rotated dimensions per
    head; values have `vdim`.  `sink`: a learned number per head joins the
    softmax denominator as exp(sink).

    The padded sizes are those the kernels work on: zeros up to a multiple of
    eight, so that every part can be read in vectors."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rotary: RotarySpec
    sink: bool = True

    @property
    def dim_p(self) -> int:
        return _pad8(self.dim)

    @property
    def rot_p(self) -> int:
        return _pad8(self.rot_dim)

    @property
    def vdim_p(self) -> int:
        return _pad8(self.vdim)

    @property
    def rank_p(self) -> int:
        return _pad8(self.kv_rank)

    @property
    def cache_width(self) -> int:
        """Cached elements of one token: the latent, then the rotated key."""
        return self.rank_p + self.rot_p

    @property
    def expand_from(self) -> int:
        """Portion length from which making all keys and values of the
        context first is less work than attending in the latent space."""
        saved = 2 * self.kv_rank - self.dim - self.vdim
        if saved <= 0:
            return 256
        # the expansion is a plain matrix product, about three times as
        # efficient as the attention work it saves
        made = self.kv_rank * (self.dim + self.vdim)
        return min(256, max(16, -(-made // (3 * saved))))


@dataclass(frozen=True)
class MlpSpec:
    """W_down gelu(W_up h) with the exact gelu, with biases or without."""
    ff: int
    bias: bool = True


@dataclass(frozen=True)
class MoeSpec:
    """Mixture of bias-free MlpSpec experts.  Each token runs the `top` ones
    with the largest sigmoid scores; the score, not renormalized, multiplies
    the expert's input.  `shared_ff`: a further expert runs for every token,
    its output multiplied by a learned sigmoid gate."""
    experts: int
    top: int
    ff: int
    shared_ff: Optional[int] = None


@dataclass(frozen=True)
class HybridLayerSpec:
    """One layer; attn and linear side by side when both are given.

    `norms`: "post", x <- norm(alpha x + y), or "sandwich",
    x <- x + norm_b(y(norm_a(x))).  Feed-forward: gated SiLU of `ff` channels,
    or what `mlp` says."""
    attn: Optional[LocalAttentionSpec] = None
    linear: Optional[LinearAttentionSpec] = None
    attn_scale: float = 1.0
    linear_scale: float = 1.0
    ff: Optional[int] = None
    kind: str = ""
    latent: Optional[LatentAttentionSpec] = None
    mlp: Optional[Union[MlpSpec, MoeSpec]] = None
    norms: str = "post"


@dataclass(frozen=True)
class LoopSpec:
    """Layers start .. stop-1 run `times` times with the same weights, each
    pass with a cache of its own; before a pass the stream becomes a linear
    map of itself and the embedding output."""
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class LayerRun:
    """One run of a layer: what it finds its cache and state under."""
    layer: int
    enter: bool = False         # the embedding output joins before it
    attn: int = -1              # index among the K/V page pools
    state: int = -1             # among the state pools
    latent: int = -1            # among the latent page pools


@dataclass(frozen=True, kw_only=True)
class HybridConfig:
    """What all hybrid architectures have."""
    name: str
    vocab_size: int
    hidden: int
    layers: Tuple[HybridLayerSpec, ...]
    rmsnorm_eps: float
    max_context: int
    max_output: int = 4096
    path: Optional[str] = None          # checkpoint folder; None: random init
    loop: Optional[LoopSpec] = None

    is_hybrid = True
    is_moe = False

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @property
    def needs_state(self) -> bool:
        return any(s.linear is not None for s in self.layers)

    def runs(self) -> List[LayerRun]:
        """The layer runs of one forward, in order."""
        order: List[Tuple[int, bool]] = [(i, False)
                                         for i in range(self.n_layers)]
        if self.loop is not None:
            lp = self.loop
            once = [(i, i == lp.start) for i in range(lp.start, lp.stop)]
            order = order[:lp.start] + once * lp.times + order[lp.stop:]
        out: List[LayerRun] = []
        attn = state = latent = 0
        for i, enter in order:
            s = self.layers[i]
            out.append(LayerRun(i, enter, attn if s.attn else -1,
                                state if s.linear else -1,
                                latent if s.latent else -1))
            attn += s.attn is not None
            state += s.linear is not None
            latent += s.latent is not None
        return out

    def run_specs(self) -> List[HybridLayerSpec]:
        return [self.layers[r.layer] for r in self.runs()]

    def kv_bytes_per_token(self, element: int = 2) -> int:
        return element * sum(
            2 * s.attn.kv_heads * s.attn.dim if s.attn else
            s.latent.cache_width if s.latent else 0 for s in self.run_specs())

    def state_bytes_per_sequence(self) -> int:
        return 4 * sum(s.linear.state_elements
                       for s in self.run_specs() if s.linear)

    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        raise NotImplementedError

    def param_count(self) -> int:
        return sum(math.prod(s) for s in self.tensor_shapes().values())


@dataclass(frozen=True, kw_only=True)
class KoridraConfig(HybridConfig):
    """Koridra: lightning layers and layers of attention beside gated linear
    attention, learned positions, norm after the sum."""
    alpha: float

    architecture = "Koridra"
    native_module = "_quoracle_hybrid"

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


# tokens a sequence may hold: the design has no position table that ends
KOTUTAR_CONTEXT = 131072


@dataclass(frozen=True, kw_only=True)
class KotutarConfig(HybridConfig):
    """Kotutar: latent attention with a sink per head, dense and
    mixture-of-experts feed-forwards, norms before and after each sublayer,
    and a run of layers that is passed through several times."""
    architecture = "Kotutar"
    native_module = "_quoracle_latent"

    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        """Checkpoint tensor names and shapes ([out, in] matrices)."""
        w = self.hidden
        t: Dict[str, Tuple[int, ...]] = {"embed": (self.vocab_size, w)}
        if self.loop is not None:
            t["loop.in"] = (w, 2 * w)
        for i, s in enumerate(self.layers):
            p, a = f"l{i}.", s.latent
            q = p + "mix."
            t.update({
                p + "norm1": (w,), p + "norm1b": (w,),
                q + "dq": (a.q_rank, w), q + "dq.norm": (a.q_rank,),
                q + "uq": (a.heads * (a.dim + a.rot_dim), a.q_rank),
                q + "dkv": (a.kv_rank + a.rot_dim, w),
                q + "dkv.norm": (a.kv_rank,),
                q + "uk": (a.heads * a.dim, a.kv_rank),
                q + "uv": (a.heads * a.vdim, a.kv_rank),
                q + "o": (w, a.heads * a.vdim)})
            if a.sink:
                t[q + "sink"] = (a.heads,)
            if s.mlp is None:
                continue
            t.update({p + "norm2": (w,), p + "norm2b": (w,)})
            p += "mlp."
            m = s.mlp
            if isinstance(m, MlpSpec):
                t.update({p + "up": (m.ff, w), p + "down": (w, m.ff)})
                if m.bias:
                    t.update({p + "up.b": (m.ff,), p + "down.b": (w,)})
                continue
            t[p + "router"] = (m.experts, w)
            for e in range(m.experts):
                t.update({f"{p}e{e}.up": (m.ff, w),
                          f"{p}e{e}.down": (w, m.ff)})
            if m.shared_ff is not None:
                t.update({p + "shared.up": (m.shared_ff, w),
                          p + "shared.down": (w, m.shared_ff),
                          p + "shared.sg": (1, w)})
        t["final.norm"] = (w,)
        t["head"] = (self.vocab_size, w)
        return t

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], name: str = "kotutar",
                  path: Optional[str] = None) -> "KotutarConfig":
        layers = tuple(_kotutar_layer(e) for e in raw["layers"])
        return cls(
            name=name, vocab_size=int(raw["vocab"]),
            hidden=int(raw["width"]), layers=layers,
            rmsnorm_eps=float(raw["norm"]["eps"]),
            loop=_loop(raw.get("loop"), len(layers)),
            max_context=KOTUTAR_CONTEXT, path=path)


def _loop(raw: Optional[Dict[str, Any]], n: int) -> Optional[LoopSpec]:
    if not raw:
        return None
    loop = LoopSpec(*(int(raw[k]) for k in ("start", "stop", "times")))
    if not 0 <= loop.start < loop.stop <= n or loop.times < 1:
        raise ValueError(f"loop {raw} does not fit {n} layers")
    return loop


def _kotutar_layer(raw: Dict[str, Any]) -> HybridLayerSpec:
    if raw["type"] != "latent_attention":
        raise ValueError(f"unknown mixer {raw['type']!r}")
    m = raw["mixer"]
    rotary = _rotary(m["rot"])
    if rotary.dims != int(m["rot_dim"]) or rotary.dims % 2:
        raise ValueError("the rotated part is rotated as a whole, in pairs: "
                         "rot.dims must be rot_dim, and even")
    latent = LatentAttentionSpec(
        heads=int(m["heads"]), dim=int(m["dim"]), rot_dim=rotary.dims,
        vdim=int(m["vdim"]), q_rank=int(m["q_rank"]),
        kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), rotary=rotary)
    return HybridLayerSpec(latent=latent, mlp=_kotutar_mlp(raw.get("mlp")),
                           norms="sandwich", kind=raw["type"])


def _kotutar_mlp(raw: Optional[Dict[str, Any]]
                 ) -> Optional[Union[MlpSpec, MoeSpec]]:
    if raw is None:
        return None
    if raw["kind"] == "dense":
        return MlpSpec(int(raw["ff"]))
    if raw["kind"] != "moe":
        raise ValueError(f"unknown feed-forward kind {raw['kind']!r}")
    router, shared = raw["router"], raw.get("shared")
    spec = MoeSpec(experts=int(router["experts"]), top=int(router["top"]),
                   ff=int(raw["expert"]["ff"]),
                   shared_ff=int(shared["ff"]) if shared else None)
    if not 1 <= spec.top <= spec.experts:
        raise ValueError(f"top {spec.top} of {spec.experts} experts")
    return spec


def kotutar_preset(name: str, *, vocab: int, hidden: int, n_layers: int,
                   ff: int, heads: int, dim: int, rot_dim: int, vdim: int,
                   q_rank: int, kv_rank: int, experts: int, top: int,
                   expert_ff: int, shared_ff: Optional[int] = None,
                   every: int = 2, loop: Optional[LoopSpec] = None,
                   max_context: int = 32768, max_output: int = 4096,
                   base: float = 500000.0) -> KotutarConfig:
    """Random-weight Kotutar: the last of every `every` layers has experts
    (0: none has)."""
    latent = LatentAttentionSpec(
        heads, dim, rot_dim, vdim, q_rank, kv_rank,
        scale=(dim + rot_dim) ** -0.5, rotary=RotarySpec(rot_dim, base))
    layers = tuple(HybridLayerSpec(
        latent=latent, norms="sandwich", kind="latent_attention",
        mlp=MoeSpec(experts, top, expert_ff, shared_ff)
        if every and i % every == every - 1 else MlpSpec(ff))
        for i in range(n_layers))
    return KotutarConfig(name=name, vocab_size=vocab, hidden=hidden,
                         layers=layers, rmsnorm_eps=1e-6, loop=loop,
                         max_context=max_context, max_output=max_output)
