"""Replay a trace of given token ids through a hosted model.

  bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come from standard input, one JSON object a line:

  {"step": 4, "entries": [{"id": "x", "tokens": [40, 7], "want": [1]}],
   "end": ["y"]}

All entries of a step are one batch of the engine (LocalEngine.step_entries:
the step, cache, state slots and kernels of generation; decode-only steps
replay the captured graphs).  `want` names places among an entry's tokens; the
logits there go to OUT/<step>.f32 (little-endian float32, [wanted, vocab], in
the order of the entries and of their places).  Requests in `end` give back
what they hold.  After each step a line "done <step>" is printed.
"""

from __future__ import annotations

import argparse
import json
import os
import sys
from typing import List, Optional, Set

STATE_SLOTS = 4             # live requests


def _native(cfg) -> None:
    """Build the model family's kernels if they are not there yet."""
    from ..ops.build import build, so_path
    if not os.path.exists(so_path(cfg.native_module)):
        build(modules=[cfg.native_module], verbose=False)


def open_engine(model: str, dtype: str, max_tokens: int,
                device: Optional[str] = None):
    import torch

    from ..engine.engine import BLOCK_SIZE, LocalEngine
    from ..models import get_config
    cfg = get_config(model)
    if device is None:
        if not torch.cuda.is_available():
            raise SystemExit("trace_run: no GPU (--device cpu runs the plain "
                             "implementations)")
        device = "cuda:0"
    if device != "cpu":
        _native(cfg)
    # float32 is true float32
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    # one block more than the tokens need: the engine's scratch block
    engine = LocalEngine(
        [model], device=torch.device(device), embed_model_key=None,
        kv_blocks_override=-(-max_tokens // BLOCK_SIZE) + 1,
        dtype=getattr(torch, dtype), state_slots=STATE_SLOTS)
    engine.precapture_graphs((1, 2, 4))
    return engine


def replay(engine, model: str, lines, out: str, say) -> None:
    live: Set[str] = set()
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = [(e["id"], e["tokens"], e.get("want", ()))
                   for e in step["entries"] if e["tokens"]]
        live.update(e[0] for e in entries)
        logits = engine.step_entries(model, entries, live) if entries else None
        if logits is not None:
            path = os.path.join(out, f"{step['step']}.f32")
            with open(path, "wb") as f:
                f.write(logits.numpy().astype("<f4").tobytes())
        for rid in step.get("end", ()):
            engine.drop_session(model, rid)
            live.discard(rid)
        say(f"done {step['step']}")


def main(argv: Optional[List[str]] = None) -> int:
    p = argparse.ArgumentParser(
        prog="trace_run", description="replay given tokens, write logits")
    p.add_argument("--model", required=True,
                   help="folder with config.json and model.safetensors")
    p.add_argument("--dtype", choices=["bfloat16", "float32"],
                   default="bfloat16")
    p.add_argument("--out", required=True, help="folder for <step>.f32")
    p.add_argument("--max-tokens", type=int, required=True,
                   help="size of the K/V pool in tokens")
    p.add_argument("--device", default=None,
                   help="cpu: the plain implementations, for tests")
    a = p.parse_args(argv)
    os.makedirs(a.out, exist_ok=True)
    engine = open_engine(a.model, a.dtype, a.max_tokens, a.device)
    replay(engine, a.model, sys.stdin, a.out,
           lambda text: print(text, flush=True))
    return 0
