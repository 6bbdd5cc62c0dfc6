"""Hybrid transformer over the HIP ops: recurrent mixers and chunk-local
attention, a float32 residual stream, norm after the sum.

Same flat-token batches as LlamaModel (decode rows first, then prefill rows),
same split of work: plain matrix products to the vendor library, everything
between them in the gfx950 kernels.  What differs:

  * the cache holds, beside K/V pages of the attention layers, one float32
    state per recurrent mixer and sequence, in slots that the session cache
    hands out;
  * every layer reads ONE fused input projection (all of its mixers' q, k, v,
    gate and decay rows); the kernels take their parts in place from its rows;
  * activations may be bf16 or float32 (`dtype`).

On the GPU the layer loop runs in the native driver (csrc/hybrid_forward.h);
the Python loop below is the CPU path and the driver's oracle.
"""

from __future__ import annotations

import os
import weakref
from typing import Callable, Dict, List, Optional, Tuple

import torch
import torch.nn.functional as F

from ..ops import hybrid as O
from ..parallel.tp import TPContext
from .checkpoint import open_checkpoint
from .config import get_config, instance_seed
from .hybrid_config import HybridLayerSpec, KoridraConfig

_ACTS = {"none": O.ACT_NONE, "silu": O.ACT_SILU, "sigmoid": O.ACT_SIGMOID}


class HybridCache:
    """K/V pages [num_blocks, kv_heads, BS, dim] of each attention layer and
    the state pool [slots + 1, heads, vdim, dim] of each recurrent mixer.  The
    last slot is scratch: padding rows of a captured decode step write there.
    A sequence that starts at position 0 starts from a zero state whatever
    its slot holds, so slots need no clearing."""

    def __init__(self, cfg: KoridraConfig, num_blocks: int, block_size: int,
                 state_slots: int, dtype: torch.dtype, device: torch.device):
        self.block_size = block_size
        self.num_blocks = num_blocks
        self.state_slots = state_slots
        self.k: List[torch.Tensor] = []
        self.v: List[torch.Tensor] = []
        self.state: List[torch.Tensor] = []
        for s in cfg.layers:
            if s.attn:
                shape = (num_blocks, s.attn.kv_heads, block_size, s.attn.dim)
                self.k.append(torch.zeros(shape, dtype=dtype, device=device))
                self.v.append(torch.zeros(shape, dtype=dtype, device=device))
            if s.linear:
                self.state.append(torch.zeros(
                    (state_slots + 1, s.linear.heads, s.linear.vdim,
                     s.linear.dim), dtype=torch.float32, device=device))

    def clear(self) -> None:
        for t in self.k + self.v + self.state:
            t.zero_()

    def bytes(self) -> int:
        return sum(t.numel() * t.element_size()
                   for t in self.k + self.v + self.state)


def _fuse(parts: List[Tuple[str, torch.Tensor]], align: int = 8
          ) -> Tuple[torch.Tensor, Dict[str, int]]:
    """Stack [out, in] matrices, each part starting at a multiple of `align`
    rows (zero rows between), so that kernels can read vectors of it."""
    rows, offsets, at = [], {}, 0
    for name, w in parts:
        offsets[name] = at
        rows.append(w)
        pad = -w.shape[0] % align
        if pad:
            rows.append(torch.zeros((pad, w.shape[1]), dtype=w.dtype,
                                    device=w.device))
        at += w.shape[0] + pad
    return torch.cat(rows).contiguous(), offsets


class HybridModel:
    """`weight(name)` gives a checkpoint tensor by name on the model's device;
    subclasses map their names onto layers."""

    def __init__(self, key: str, device: torch.device,
                 dtype: torch.dtype = torch.bfloat16,
                 cfg: Optional[KoridraConfig] = None,
                 tp: Optional[TPContext] = None):
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("hybrid models run in bfloat16 or float32")
        if tp is not None and tp.world > 1:
            raise NotImplementedError(
                "hybrid models do not shard over a tensor-parallel group; "
                "place whole models on ranks instead")
        self.key = key
        self.cfg = cfg or get_config(key)
        self.device = device
        self.dtype = dtype
        # per layer: tensors and numbers, in the native driver's names
        self.tensors: List[Dict[str, torch.Tensor]] = []
        self.numbers: List[Dict[str, float]] = []
        self.embed = self.head = self.final_norm = None
        self.pos: Optional[torch.Tensor] = None
        self._n_attn = self._n_state = 0
        self._load(self._source())
        self._register_native()

    # -- weights -------------------------------------------------------------

    def _source(self) -> Callable[[str], torch.Tensor]:
        """weight(name) from the checkpoint folder, or random weights that
        depend only on the model key."""
        shapes = self.cfg.tensor_shapes()
        if self.cfg.path is not None:
            ckpt = open_checkpoint(self.cfg.path)

            def read(name: str) -> torch.Tensor:
                got = ckpt.shape(name)
                want = shapes[name]
                if len(got) != len(want) or any(
                        w and g != w for g, w in zip(got, want)):
                    raise ValueError(f"{name}: shape {got}, expected {want}")
                return ckpt.get(name).to(self.device)
            return read

        gen_dev = "cpu" if self.cfg.hidden <= 1024 or \
            self.device.type == "cpu" else self.device
        gen = torch.Generator(device=gen_dev)
        gen.manual_seed(instance_seed(self.key))

        def draw(name: str) -> torch.Tensor:
            shape = shapes[name]
            if name.rsplit(".", 1)[-1] in ("norm", "norm1", "norm2"):
                return torch.ones(shape, device=self.device)
            w = torch.empty(shape, device=gen_dev)
            w.normal_(0.0, 0.02 if len(shape) > 1 else 1.0, generator=gen)
            return w.to(self.dtype).to(self.device)
        return draw

    def _load(self, weight: Callable[[str], torch.Tensor]) -> None:
        raise NotImplementedError

    def _mat(self, w: torch.Tensor) -> torch.Tensor:
        return w.to(self.dtype).contiguous()

    @staticmethod
    def _f32(w: torch.Tensor) -> torch.Tensor:
        return w.float().contiguous()

    def _add_layer(self, spec: HybridLayerSpec, norm1: torch.Tensor,
                   attn: Dict[str, torch.Tensor],
                   linear: Dict[str, torch.Tensor],
                   mlp: Dict[str, torch.Tensor]) -> None:
        """Fuse one layer's named weights into what the kernels read.
        attn: q k o q.norm k.norm; linear: q k v g o norm (a1 a2 a2.b);
        mlp: gate up down norm (empty when there is none)."""
        parts: List[Tuple[str, torch.Tensor]] = []
        if spec.attn:
            parts += [("attn." + n, attn[n]) for n in ("q", "k")]
        if spec.linear:
            names = ["q", "k", "v", "g"]
            if spec.linear.decay is None:
                names.append("a1")
            parts += [("lin." + n, linear[n]) for n in names]
        w_in, off = _fuse([(n, self._mat(w)) for n, w in parts])
        t: Dict[str, torch.Tensor] = {"w_in": w_in, "norm1": self._f32(norm1)}
        n: Dict[str, float] = {}
        if spec.attn:
            a = spec.attn
            freq, mag = a.rotary.frequencies() if a.rotary else ((), 1.0)
            t["attn.q_norm"] = self._f32(attn["q.norm"])
            t["attn.k_norm"] = self._f32(attn["k.norm"])
            t["attn.freq"] = torch.tensor(freq, dtype=torch.float64,
                                          device=self.device)
            t["attn.w_o"] = self._mat(attn["o"])
            n.update({"attn.q_off": off["attn.q"],
                      "attn.k_off": off["attn.k"],
                      "attn.heads": a.heads, "attn.dim": a.dim,
                      "attn.chunk": a.chunk, "attn.scale": a.scale,
                      "attn.mag": mag, "attn.sink": float(a.sink),
                      "attn.out_scale": spec.attn_scale,
                      "attn.cache": self._n_attn})
            self._n_attn += 1
        if spec.linear:
            lin = spec.linear
            t["lin.w_o"] = self._mat(linear["o"])
            t["lin.norm"] = self._f32(linear["norm"])
            n.update({"lin." + p + "_off": off["lin." + p] for p in "qkvg"})
            n.update({"lin.heads": lin.heads, "lin.vdim": lin.vdim,
                      "lin.act": _ACTS[lin.act],
                      "lin.gate_act": _ACTS[lin.gate_act],
                      "lin.groups": lin.heads if lin.head_norm else 1,
                      "lin.qscale": lin.qscale,
                      "lin.channel": float(lin.decay is None),
                      "lin.out_scale": spec.linear_scale,
                      "lin.state": self._n_state})
            self._n_state += 1
            if lin.decay is None:
                t["lin.a2"] = self._mat(linear["a2"])
                t["lin.a2_b"] = self._f32(linear["a2.b"])
                n["lin.a_off"] = off["lin.a1"]
                n["lin.tau"] = lin.tau
            else:
                d = torch.tensor(lin.decay, dtype=torch.float64)
                steps = torch.arange(O.LIN_CHUNK + 1, dtype=torch.float64)
                t["lin.decay"] = d.float().to(self.device)
                t["lin.powers"] = (d[:, None] ** steps[None, :]).float() \
                    .contiguous().to(self.device)
        if spec.ff is not None:
            t["gate_up"] = torch.cat([self._mat(mlp["gate"]),
                                      self._mat(mlp["up"])]).contiguous()
            t["down"] = self._mat(mlp["down"])
            t["norm2"] = self._f32(mlp["norm"])
        self.tensors.append(t)
        self.numbers.append(n)

    def _register_native(self) -> None:
        self.use_cpp = False
        if self.device.type != "cuda" or \
                os.environ.get("QUORACLE_NO_CPP_FWD"):
            return
        from .. import ops
        ext = ops.hybrid_ext()          # raises when the kernels are missing
        self._handle = f"{self.key}@{id(self)}"
        top = {"embed": self.embed, "head": self.head,
               "final_norm": self.final_norm}
        if self.pos is not None:
            top["pos"] = self.pos
        ext.register_hybrid(self._handle, top,
                            {"alpha": self.cfg.alpha,
                             "eps": self.cfg.rmsnorm_eps},
                            self.tensors, self.numbers)
        weakref.finalize(self, ext.unregister_hybrid, self._handle)
        self.use_cpp = True

    def param_bytes(self) -> int:
        tensors = [self.embed, self.head, self.final_norm]
        if self.pos is not None:
            tensors.append(self.pos)
        for t in self.tensors:
            tensors += list(t.values())
        return sum(t.numel() * t.element_size() for t in tensors)

    def new_kv_cache(self, num_blocks: int, block_size: int,
                     state_slots: int = 1) -> HybridCache:
        return HybridCache(self.cfg, num_blocks, block_size, state_slots,
                           self.dtype, self.device)

    # -- forward -------------------------------------------------------------

    def forward(self, batch, kv: HybridCache,
                stream: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
        """The float32 residual stream [T, hidden] after the last layer.
        `stream`, when given, collects it after every layer (this takes the
        Python loop)."""
        if self.use_cpp and stream is None:
            from .. import ops
            return ops.hybrid_ext().hybrid_forward(
                self._handle, batch.hybrid_tensors(), batch.n_decode,
                batch.max_ctx, batch.max_kv, kv.k, kv.v, kv.state)
        cfg, dev = self.cfg, self.device
        T = batch.total_tokens
        x = torch.empty((T, cfg.hidden), dtype=torch.float32, device=dev)
        h = torch.empty((T, cfg.hidden), dtype=self.dtype, device=dev)
        O.embed_positions(x, h, self.embed, self.pos, batch.tokens,
                          batch.positions)
        for t, n in zip(self.tensors, self.numbers):
            proj = F.linear(h, t["w_in"])
            mixed: List[Tuple[torch.Tensor, float]] = []
            if "attn.w_o" in t:
                mixed.append((self._attention(t, n, proj, batch, kv),
                              n["attn.out_scale"]))
            if "lin.w_o" in t:
                mixed.append((self._linear(t, n, proj, batch, kv),
                              n["lin.out_scale"]))
            second = mixed[1] if len(mixed) > 1 else (None, 0.0)
            O.post_norm(x, h, *mixed[0], *second, cfg.alpha, t["norm1"],
                        cfg.rmsnorm_eps)
            if "gate_up" in t:
                gu = F.linear(h, t["gate_up"])
                act = torch.empty((T, gu.shape[1] // 2), dtype=self.dtype,
                                  device=dev)
                O.glu(act, gu)
                O.post_norm(x, h, F.linear(act, t["down"]), 1.0, None, 0.0,
                            cfg.alpha, t["norm2"], cfg.rmsnorm_eps)
            if stream is not None:
                stream.append(x.clone())
        return x

    def _attention(self, t, n, proj, batch, kv) -> torch.Tensor:
        T, H, D = proj.shape[0], int(n["attn.heads"]), int(n["attn.dim"])
        kc, vc = kv.k[int(n["attn.cache"])], kv.v[int(n["attn.cache"])]
        q = torch.empty((T, H, D), dtype=self.dtype, device=self.device)
        out = torch.empty_like(q)
        O.qk_norm_rope_store(q, kc, vc, proj, n["attn.q_off"],
                             n["attn.k_off"], t["attn.q_norm"],
                             t["attn.k_norm"], batch.positions, batch.slots,
                             t["attn.freq"], n["attn.mag"],
                             self.cfg.rmsnorm_eps)
        O.local_attention(out, q, kc, vc, batch, n["attn.scale"],
                          int(n["attn.chunk"]), bool(n["attn.sink"]))
        return F.linear(out.view(T, H * D), t["attn.w_o"])

    def _linear(self, t, n, proj, batch, kv) -> torch.Tensor:
        T, dev = proj.shape[0], self.device
        state = kv.state[int(n["lin.state"])]
        channel = bool(n["lin.channel"])
        o = torch.empty((T, int(n["lin.heads"]) * int(n["lin.vdim"])),
                        dtype=self.dtype, device=dev)
        decay = t.get("lin.decay")
        if channel:
            decay = torch.empty((T, t["lin.a2"].shape[0]),
                                dtype=torch.float32, device=dev)
            O.log_decay(decay, proj, int(n["lin.a_off"]), t["lin.a2"],
                        t["lin.a2_b"], n["lin.tau"], batch, state)
        O.linear_attention(o, proj, n["lin.q_off"], n["lin.k_off"],
                           n["lin.v_off"], n["lin.act"], n["lin.qscale"],
                           decay, t.get("lin.powers"), channel, state, batch)
        gated = torch.empty_like(o)
        O.gated_norm(gated, o, proj, n["lin.g_off"], t["lin.norm"],
                     n["lin.groups"], n["lin.gate_act"],
                     self.cfg.rmsnorm_eps)
        return F.linear(gated, t["lin.w_o"])

    def compute_logits(self, x: torch.Tensor,
                       rows: torch.Tensor) -> torch.Tensor:
        """Final norm and head of the rows that need them: [R, vocab] f32."""
        if self.use_cpp:
            from .. import ops
            return ops.hybrid_ext().hybrid_logits(self._handle, x, rows)
        h = torch.empty((rows.shape[0], x.shape[1]), dtype=self.dtype,
                        device=self.device)
        O.norm_rows(h, x, rows, self.final_norm, self.cfg.rmsnorm_eps)
        return F.linear(h, self.head).float()


class KoridraModel(HybridModel):
    def _load(self, weight: Callable[[str], torch.Tensor]) -> None:
        self.embed = self._mat(weight("embed"))
        self.pos = self._mat(weight("pos"))
        for i, spec in enumerate(self.cfg.layers):
            p = f"l{i}."
            ap, lp = ((p + "mix.left.", p + "mix.right.") if spec.attn
                      else ("", p + "mix."))
            attn = {n: weight(ap + n)
                    for n in ("q", "k", "q.norm", "k.norm", "o")} \
                if spec.attn else {}
            names = ["q", "k", "v", "g", "o", "norm"]
            if spec.linear.decay is None:
                names += ["a1", "a2", "a2.b"]
            mlp = {}
            if spec.ff is not None:
                mlp = {n: weight(p + "mlp." + n)
                       for n in ("gate", "up", "down")}
                mlp["norm"] = weight(p + "norm2")
            self._add_layer(spec, weight(p + "norm1"), attn,
                            {n: weight(lp + n) for n in names}, mlp)
        self.final_norm = self._f32(weight("final.norm"))
        self.head = self._mat(weight("head"))
