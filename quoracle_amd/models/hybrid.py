"""Hybrid transformer over the HIP ops: recurrent mixers, chunk-local
attention and attention over cached latents, dense and mixture-of-experts
feed-forwards, a float32 residual stream.

Same flat-token batches as LlamaModel (decode rows first, then prefill rows),
same split of work: plain matrix products to the vendor library, everything
between them in the gfx950 kernels.  What differs:

  * the cache holds, beside K/V pages of the attention layers, pages of
    latents, and one float32 state per recurrent mixer and sequence, in slots
    that the session cache hands out;
  * a forward is a list of layer runs: a layer that is passed through several
    times has a cache of its own for each pass;
  * every layer reads ONE fused input projection (all rows that its mixers
    take from the layer's input); the kernels take their parts in place;
  * norms sit after the residual sum, or before and after each sublayer;
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
from ..ops import latent as L
from ..parallel.tp import TPContext
from .checkpoint import open_checkpoint
from .config import get_config, instance_seed
from .hybrid_config import (HybridConfig, HybridLayerSpec,
                            LatentAttentionSpec, MlpSpec, MoeSpec)

_ACTS = {"none": O.ACT_NONE, "silu": O.ACT_SILU, "sigmoid": O.ACT_SIGMOID}


class HybridCache:
    """K/V pages [num_blocks, kv_heads, BS, dim] of each run of an attention
    layer, pages of latents [num_blocks, BS, width] of each run of a latent
    attention layer, and the state pool [slots + 1, heads, vdim, dim] of each
    run of a recurrent mixer.  The last slot is scratch: padding rows of a
    captured decode step write there.  A sequence that starts at position 0
    starts from a zero state whatever its slot holds, so slots need no
    clearing."""

    def __init__(self, cfg: HybridConfig, num_blocks: int, block_size: int,
                 state_slots: int, dtype: torch.dtype, device: torch.device):
        self.block_size = block_size
        self.num_blocks = num_blocks
        self.state_slots = state_slots if cfg.needs_state else 0
        self.k: List[torch.Tensor] = []
        self.v: List[torch.Tensor] = []
        self.state: List[torch.Tensor] = []
        self.latent: List[torch.Tensor] = []
        for s in cfg.run_specs():
            if s.attn:
                shape = (num_blocks, s.attn.kv_heads, block_size, s.attn.dim)
                self.k.append(torch.zeros(shape, dtype=dtype, device=device))
                self.v.append(torch.zeros(shape, dtype=dtype, device=device))
            if s.linear:
                self.state.append(torch.zeros(
                    (state_slots + 1, s.linear.heads, s.linear.vdim,
                     s.linear.dim), dtype=torch.float32, device=device))
            if s.latent:
                self.latent.append(torch.zeros(
                    (num_blocks, block_size, s.latent.cache_width),
                    dtype=dtype, device=device))

    def pools(self) -> Dict[str, List[torch.Tensor]]:
        return {"k": self.k, "v": self.v, "state": self.state,
                "latent": self.latent}

    def clear(self) -> None:
        for pool in self.pools().values():
            for t in pool:
                t.zero_()

    def bytes(self) -> int:
        return sum(t.numel() * t.element_size()
                   for pool in self.pools().values() for t in pool)


def _pad_rows(w: torch.Tensor, groups: int, parts: List[Tuple[int, int]]
              ) -> torch.Tensor:
    """[groups * sum(n), in] -> each part of n rows of a group padded with
    zero rows to its second size."""
    w = w.view(groups, sum(n for n, _ in parts), -1)
    out, at = [], 0
    for n, size in parts:
        out.append(F.pad(w[:, at:at + n], (0, 0, 0, size - n)))
        at += n
    return torch.cat(out, 1).flatten(0, 1)


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
                 cfg: Optional[HybridConfig] = None,
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
        self.loop_in: Optional[torch.Tensor] = None
        self.alpha = 1.0
        self.runs = self.cfg.runs()
        self._load(self._source())
        self.expand_from = self._expand_from()
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
            if name.rsplit(".", 1)[-1] in ("norm", "norm1", "norm2", "norm1b",
                                           "norm2b"):
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
                      "attn.out_scale": spec.attn_scale})
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
                      "lin.out_scale": spec.linear_scale})
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

    def _add_sandwich_layer(self, spec: HybridLayerSpec,
                            norms: Dict[str, torch.Tensor],
                            latent: Dict[str, torch.Tensor],
                            mlp: Dict[str, torch.Tensor]) -> None:
        """A layer of latent attention with norms before and after each
        sublayer.  norms: norm1 norm1b (norm2 norm2b); latent: dq dq.norm uq
        dkv dkv.norm uk uv o (sink); mlp: up down (up.b down.b), or with
        experts router e.up e.down (shared.up shared.down shared.sg)."""
        t = {k: self._f32(w) for k, w in norms.items()}
        n: Dict[str, float] = {}
        self._put_latent(t, n, spec.latent, latent)
        if isinstance(spec.mlp, MlpSpec):
            t["mlp.up"], t["mlp.down"] = (self._mat(mlp[k])
                                          for k in ("up", "down"))
            if spec.mlp.bias:
                t["mlp.up_b"], t["mlp.down_b"] = (
                    self._f32(mlp[k]) for k in ("up.b", "down.b"))
        elif isinstance(spec.mlp, MoeSpec):
            shared = spec.mlp.shared_ff is not None
            # the shared expert's gate is one more row of the router
            t["moe.router"] = self._mat(torch.cat(
                [mlp["router"]] + ([mlp["shared.sg"]] if shared else [])))
            t["moe.up"], t["moe.down"] = (self._mat(mlp[k])
                                          for k in ("e.up", "e.down"))
            if shared:
                t["moe.shared_up"], t["moe.shared_down"] = (
                    self._mat(mlp[k]) for k in ("shared.up", "shared.down"))
            n["moe.top"] = spec.mlp.top
        self.tensors.append(t)
        self.numbers.append(n)

    def _put_latent(self, t: Dict[str, torch.Tensor], n: Dict[str, float],
                    a: LatentAttentionSpec,
                    w: Dict[str, torch.Tensor]) -> None:
        w_in, off = _fuse([(k, self._mat(w[k])) for k in ("dq", "dkv")])
        freq, mag = a.rotary.frequencies()
        if mag != 1.0:
            raise ValueError("latent attention rotates without a factor")
        rank = (0, a.rank_p - a.kv_rank)
        uk = F.pad(_pad_rows(self._mat(w["uk"]), a.heads,
                             [(a.dim, a.dim_p)]), rank)
        uv = F.pad(_pad_rows(self._mat(w["uv"]), a.heads,
                             [(a.vdim, a.vdim_p)]), rank)
        # keys and values of a token from its latent: every head's key rows,
        # then every head's value rows
        t["lat.w_kv"] = torch.cat([uk, uv]).contiguous()
        # queries into the latent space
        t["lat.w_uk_t"] = uk.view(a.heads, a.dim_p, a.rank_p) \
            .transpose(1, 2).contiguous()
        t["lat.w_in"] = w_in
        t["lat.w_uq"] = _pad_rows(
            self._mat(w["uq"]), a.heads,
            [(a.dim, a.dim_p), (a.rot_dim, a.rot_p)]).contiguous()
        t["lat.w_o"] = F.pad(
            self._mat(w["o"]).view(-1, a.heads, a.vdim),
            (0, a.vdim_p - a.vdim)).flatten(1).contiguous()
        t["lat.q_norm"] = self._f32(w["dq.norm"])
        t["lat.kv_norm"] = self._f32(w["dkv.norm"])
        t["lat.freq"] = torch.tensor(freq, dtype=torch.float64,
                                     device=self.device)
        if a.sink:
            t["lat.sink"] = self._f32(w["sink"])
        n.update({"lat.heads": a.heads, "lat.dim": a.dim_p,
                  "lat.rot": a.rot_p, "lat.vdim": a.vdim_p,
                  "lat.rank": a.rank_p, "lat.kv_off": off["dkv"],
                  "lat.scale": a.scale})

    def _expand_from(self) -> Optional[int]:
        """Portions of at least this many tokens attend over expanded keys
        and values, shorter ones in the latent space; None: the model makes
        no such difference."""
        specs = [s.latent for s in self.cfg.layers if s.latent]
        if not specs or self.device.type != "cuda" or not all(
                L.tiles_ok(s, self.dtype) for s in specs):
            return None
        if not all(L.expandable(s) for s in specs):
            return 1 << 30
        return max(s.expand_from for s in specs)

    def _register_native(self) -> None:
        self.use_cpp = False
        if self.device.type != "cuda" or \
                os.environ.get("QUORACLE_NO_CPP_FWD"):
            return
        from .. import ops
        # raises when the kernels are missing
        ext = self._ext = ops.module(self.cfg.native_module)
        self._handle = f"{self.key}@{id(self)}"
        top = {"embed": self.embed, "head": self.head,
               "final_norm": self.final_norm}
        if self.pos is not None:
            top["pos"] = self.pos
        if self.loop_in is not None:
            top["loop_in"] = self.loop_in
        ext.register_model(
            self._handle, top,
            {"alpha": self.alpha, "eps": self.cfg.rmsnorm_eps},
            self.tensors, self.numbers,
            [{"layer": r.layer, "enter": int(r.enter), "attn": r.attn,
              "state": r.state, "latent": r.latent} for r in self.runs])
        weakref.finalize(self, ext.unregister_model, self._handle)
        self.use_cpp = True

    def param_bytes(self) -> int:
        tensors = [self.embed, self.head, self.final_norm]
        tensors += [t for t in (self.pos, self.loop_in) if t is not None]
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
        `stream`, when given, collects it after every layer run (this takes
        the Python loop)."""
        if self.use_cpp and stream is None:
            return self._ext.forward(
                self._handle, batch.hybrid_tensors(), batch.hybrid_numbers(),
                kv.pools())
        cfg, dev = self.cfg, self.device
        T = batch.total_tokens
        x = torch.empty((T, cfg.hidden), dtype=torch.float32, device=dev)
        h = torch.empty((T, cfg.hidden), dtype=self.dtype, device=dev)
        O.embed_positions(x, h, self.embed, self.pos, batch.tokens,
                          batch.positions)
        # [stream, embedding output], the input of a pass
        joined = torch.cat([h, h], 1) if self.loop_in is not None else None
        for i, run in enumerate(self.runs):
            t, n = self.tensors[run.layer], self.numbers[run.layer]
            spec = cfg.layers[run.layer]
            if spec.norms == "sandwich":
                if run.enter:
                    L.pre_norm(x, h, L.linear_f32(joined, self.loop_in),
                               t["norm1"], cfg.rmsnorm_eps)
                elif i == 0:
                    L.pre_norm(x, h, None, t["norm1"], cfg.rmsnorm_eps)
                self._sandwich_layer(t, n, run, spec, batch, kv, x, h, joined,
                                     self._next_norm(i))
            else:
                self._post_layer(t, n, run, batch, kv, x, h)
            if stream is not None:
                stream.append(x.clone())
        return x

    def _next_norm(self, i: int) -> Tuple[Optional[torch.Tensor], bool]:
        """(the norm that the stream goes through after run i, whether the
        embedding output joins instead)."""
        if i + 1 == len(self.runs):
            return None, False
        run = self.runs[i + 1]
        if run.enter:
            return None, True
        return self.tensors[run.layer]["norm1"], False

    def _post_layer(self, t, n, run, batch, kv, x, h) -> None:
        cfg = self.cfg
        proj = F.linear(h, t["w_in"])
        mixed: List[Tuple[torch.Tensor, float]] = []
        if "attn.w_o" in t:
            mixed.append((self._attention(t, n, run, proj, batch, kv),
                          n["attn.out_scale"]))
        if "lin.w_o" in t:
            mixed.append((self._linear(t, n, run, proj, batch, kv),
                          n["lin.out_scale"]))
        second = mixed[1] if len(mixed) > 1 else (None, 0.0)
        O.post_norm(x, h, *mixed[0], *second, self.alpha, t["norm1"],
                    cfg.rmsnorm_eps)
        if "gate_up" in t:
            gu = F.linear(h, t["gate_up"])
            act = torch.empty((h.shape[0], gu.shape[1] // 2),
                              dtype=self.dtype, device=self.device)
            O.glu(act, gu)
            O.post_norm(x, h, F.linear(act, t["down"]), 1.0, None, 0.0,
                        self.alpha, t["norm2"], cfg.rmsnorm_eps)

    def _sandwich_layer(self, t, n, run, spec, batch, kv, x, h, joined,
                        after) -> None:
        eps = self.cfg.rmsnorm_eps
        # the norm that h goes through next; or where the stream goes instead
        last = (x, h, joined if after[1] else None, after[0])
        y = self._latent(t, n, run, h, batch, kv)
        if spec.mlp is None:
            L.sandwich_norm(*last, y, None, None, None, t["norm1b"], eps)
            return
        L.sandwich_norm(x, h, None, t["norm2"], y, None, None, None,
                        t["norm1b"], eps)
        if "mlp.up" in t:
            y, bias = self._mlp(t, h), t.get("mlp.down_b")
            L.sandwich_norm(*last, y, bias, None, None, t["norm2b"], eps)
        else:
            y, shared, gate = self._moe(t, n, h)
            L.sandwich_norm(*last, y, None, shared, gate, t["norm2b"], eps)

    def _latent(self, t, n, run, h, batch, kv) -> torch.Tensor:
        T, H = h.shape[0], int(n["lat.heads"])
        pool = kv.latent[run.latent]
        proj = F.linear(h, t["lat.w_in"])
        cq = torch.empty((T, t["lat.q_norm"].shape[0]), dtype=self.dtype,
                         device=self.device)
        L.latent_store(cq, pool, proj, int(n["lat.kv_off"]),
                       int(n["lat.rank"]), t["lat.q_norm"], t["lat.kv_norm"],
                       batch.positions, batch.slots, t["lat.freq"],
                       self.cfg.rmsnorm_eps)
        q = F.linear(cq, t["lat.w_uq"]).view(T, H, -1)
        L.rotate_heads(q, int(n["lat.dim"]), batch.positions, t["lat.freq"])
        out = torch.empty((T, H, int(n["lat.vdim"])), dtype=self.dtype,
                          device=self.device)
        L.latent_attention(out, q, pool, t["lat.w_kv"], t["lat.w_uk_t"],
                           t.get("lat.sink"), n["lat.scale"], batch)
        return F.linear(out.flatten(1), t["lat.w_o"])

    def _mlp(self, t, h, name: str = "mlp.") -> torch.Tensor:
        up = F.linear(h, t[name + "up"])
        L.bias_gelu(up, t.get(name + "up_b"))
        return F.linear(up, t[name + "down"])

    def _moe(self, t, n, h):
        """([T, top, hidden] outputs of the chosen experts, shared expert's
        output, its gate)."""
        T, top = h.shape[0], int(n["moe.top"])
        E = t["moe.up"].shape[0]
        ids = torch.empty((T, top), dtype=torch.int32, device=self.device)
        weights = torch.empty((T, top), dtype=torch.float32,
                              device=self.device)
        shared = gate = None
        if "moe.shared_up" in t:
            gate = torch.empty(T, dtype=torch.float32, device=self.device)
        L.moe_route(ids, weights, gate, h, t["moe.router"], E)
        if gate is not None:
            shared = self._mlp(t, h, "moe.shared_")
        y = torch.empty((T, top, h.shape[1]), dtype=self.dtype,
                        device=self.device)
        L.moe_experts(y, h, ids, weights, t["moe.up"], t["moe.down"])
        return y, shared, gate

    def _attention(self, t, n, run, proj, batch, kv) -> torch.Tensor:
        T, H, D = proj.shape[0], int(n["attn.heads"]), int(n["attn.dim"])
        kc, vc = kv.k[run.attn], kv.v[run.attn]
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

    def _linear(self, t, n, run, proj, batch, kv) -> torch.Tensor:
        T, dev = proj.shape[0], self.device
        state = kv.state[run.state]
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
            return self._ext.logits(self._handle, x, rows)
        h = torch.empty((rows.shape[0], x.shape[1]), dtype=self.dtype,
                        device=self.device)
        O.norm_rows(h, x, rows, self.final_norm, self.cfg.rmsnorm_eps)
        return F.linear(h, self.head).float()


class KoridraModel(HybridModel):
    def _load(self, weight: Callable[[str], torch.Tensor]) -> None:
        self.alpha = self.cfg.alpha
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


class KotutarModel(HybridModel):
    def _load(self, weight: Callable[[str], torch.Tensor]) -> None:
        self.embed = self._mat(weight("embed"))
        if self.cfg.loop is not None:
            self.loop_in = self._mat(weight("loop.in"))
        for i, spec in enumerate(self.cfg.layers):
            p = f"l{i}."
            names = ["dq", "dq.norm", "uq", "dkv", "dkv.norm", "uk", "uv",
                     "o"] + (["sink"] if spec.latent.sink else [])
            norms = ["norm1", "norm1b"] + (["norm2", "norm2b"]
                                           if spec.mlp else [])
            self._add_sandwich_layer(
                spec, {k: weight(p + k) for k in norms},
                {k: weight(p + "mix." + k) for k in names},
                self._feed_forward(spec, p + "mlp.", weight))
        self.final_norm = self._f32(weight("final.norm"))
        self.head = self._mat(weight("head"))

    def _feed_forward(self, spec: HybridLayerSpec, p: str,
                      weight: Callable[[str], torch.Tensor]
                      ) -> Dict[str, torch.Tensor]:
        m = spec.mlp
        if m is None:
            return {}
        if isinstance(m, MlpSpec):
            names = ["up", "down"] + (["up.b", "down.b"] if m.bias else [])
        else:
            names = ["router"]
            if m.shared_ff is not None:
                names += ["shared.up", "shared.down", "shared.sg"]
        out = {k: weight(p + k) for k in names}
        if isinstance(m, MoeSpec):
            for k in ("up", "down"):
                # filled expert by expert: no second copy of all of them
                first = weight(f"{p}e0.{k}")
                stack = torch.empty((m.experts, *first.shape),
                                    dtype=self.dtype, device=self.device)
                for e in range(m.experts):
                    stack[e] = first if e == 0 else weight(f"{p}e{e}.{k}")
                out["e." + k] = stack
        return out
