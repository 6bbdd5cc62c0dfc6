"""Prefill and decode throughput of the hybrid models beside Llama-family
models of equal size, through the engine's own step.

  python bench.py --layer-bench            (one JSON line per measurement)

Random weights; a few layers of the size of a 1B-class and of an 8B-class
model, so that a step is long enough to time and short enough to repeat.  The
models take turns.  Beside Llama stand Koridra and Kotutar with dense
feed-forwards, beside Mixtral (Llama with experts) Kotutar with experts.
Kotutar's feed-forwards have two matrices for Llama's three and are as much
wider.
"""

from __future__ import annotations

import json
import sys
import time
from dataclasses import replace
from typing import Dict, List

import torch

# name -> (hidden, ff, layers, heads, kv heads, head dim)
SIZES = {
    "1b-layers": (2048, 8192, 8, 16, 4, 128),
    "8b-layers": (4096, 14336, 8, 32, 8, 128),
}
EXPERTS, TOP = 8, 2
VOCAB = 32000
CONTEXT = 16384
ATTN_CHUNK = 8192


def configs(size: str) -> Dict[str, object]:
    from ..models.config import PRESETS
    from ..models.hybrid_config import koridra_preset, kotutar_preset
    hidden, ff, layers, heads, kv, dim = SIZES[size]
    llama = replace(PRESETS["llama3-8b"], name=f"llama-{size}",
                    vocab_size=VOCAB, n_layers=layers, hidden=hidden,
                    n_heads=heads, n_kv_heads=kv, head_dim=dim,
                    intermediate=ff, max_context=CONTEXT)

    def kotutar(name: str, every: int):
        return kotutar_preset(
            f"{name}-{size}", vocab=VOCAB, hidden=hidden, n_layers=layers,
            ff=ff * 3 // 2, heads=heads, dim=dim, rot_dim=dim // 2, vdim=dim,
            q_rank=hidden * 3 // 8, kv_rank=512, experts=EXPERTS, top=TOP,
            expert_ff=ff * 3 // 2, every=every, max_context=CONTEXT)
    return {
        "llama": llama,
        "koridra": koridra_preset(
            f"koridra-{size}", vocab=VOCAB, hidden=hidden, n_layers=layers,
            ff=ff, heads=heads, kv_heads=kv, dim=dim, chunk=ATTN_CHUNK,
            lin_heads=heads, lin_dim=dim, lin_vdim=dim, max_context=CONTEXT),
        "kotutar": kotutar("kotutar", 0),
        "mixtral": replace(llama, name=f"mixtral-{size}", n_experts=EXPERTS,
                           top_k_experts=TOP),
        "kotutar-moe": kotutar("kotutar-moe", 1),
    }


class Side:
    """One hosted model and its running sequences."""

    def __init__(self, name: str, cfg, device: torch.device, batch: int):
        from ..engine.engine import LocalEngine
        from ..models.config import PRESETS
        self.name, self.key = name, cfg.name
        PRESETS[cfg.name] = cfg
        self.engine = LocalEngine(
            [cfg.name], device=device, embed_model_key=None,
            kv_blocks_override=(batch + 1) * CONTEXT // 16 // 2 + 64,
            state_slots=batch + 1)
        self.params = self.engine.models[self.key].model.param_bytes() // 2

    def feed(self, entries) -> None:
        self.engine.step_entries(self.key, entries,
                                 live=[e[0] for e in entries])

    def drop(self, ids: List[str]) -> None:
        for i in ids:
            self.engine.drop_session(self.key, i)


def _sync(device: torch.device) -> None:
    if device.type == "cuda":
        torch.cuda.synchronize(device)


def _timed(device, fn) -> float:
    _sync(device)
    t0 = time.perf_counter()
    fn()
    _sync(device)
    return time.perf_counter() - t0


def prefill(sides: List[Side], device, tokens: int, before: int,
            repeats: int = 5) -> Dict[str, float]:
    """Seconds to prefill `tokens` behind `before` cached ones (best)."""
    best = {s.name: float("inf") for s in sides}
    piece = [(7 * i) % VOCAB for i in range(tokens)]
    for turn in range(repeats + 1):
        for s in sides:
            for at in range(0, before, 2048):
                s.feed([("p", piece[:1] * min(2048, before - at), ())])
            dt = _timed(device, lambda: s.feed([("p", piece, ())]))
            if turn:
                best[s.name] = min(best[s.name], dt)
            s.drop(["p"])
    return best


def decode(sides: List[Side], device, batch: int, context: int,
           steps: int = 64) -> Dict[str, float]:
    """Seconds per decode step of `batch` sequences around `context`."""
    best = {s.name: float("inf") for s in sides}
    ids = [f"d{i}" for i in range(batch)]
    for s in sides:
        for i in ids:
            for at in range(0, context, 2048):
                s.feed([(i, [3] * min(2048, context - at), ())])
    for turn in range(3):
        for s in sides:
            s.feed([(i, [5], ()) for i in ids])

            def run():
                # a different token for each, so that experts differ too
                for t in range(steps):
                    s.feed([(i, [(131 * t + 977 * k) % VOCAB], ())
                            for k, i in enumerate(ids)])
            best[s.name] = min(best[s.name], _timed(device, run) / steps)
    for s in sides:
        s.drop(ids)
    return best


def main(sizes=tuple(SIZES), batches=(1, 16, 64), device=None,
         only=None) -> None:
    device = torch.device(device or "cuda:0")
    for size in sizes:
        # interleave: all models live on the GPU at once
        sides = [Side(n, c, device, max(batches))
                 for n, c in configs(size).items() if not only or n in only]
        for s in sides:
            s.engine.precapture_graphs(tuple(batches))

        def report(metric: str, seconds: Dict[str, float], tokens: int,
                   **what) -> None:
            for s in sides:
                print(json.dumps({
                    "metric": metric, "model": s.key, "unit": "tokens/s",
                    "value": round(tokens / seconds[s.name], 1),
                    "ms_per_step": round(seconds[s.name] * 1e3, 3),
                    "params_m": round(s.params / 1e6), "dtype": "bf16",
                    "data": "synthetic, random weights", **what}), flush=True)

        for tokens, before in ((2048, 0), (2048, 4096), (8192, 0), (64, 4096)):
            report("prefill", prefill(sides, device, tokens, before), tokens,
                   new_tokens=tokens, cached_tokens=before)
        for b in batches:
            report("decode", decode(sides, device, b, 4000), b, batch=b,
                   context=4000)
        del sides
        print(f"[layer-bench] {size} done", file=sys.stderr, flush=True)
        if device.type == "cuda":
            torch.cuda.empty_cache()
