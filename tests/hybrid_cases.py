"""What the tests of all hybrid models share: a random model on disk, helpers
that feed it to the engine, and the comparison with its plain oracle."""

import json
import os
import struct

import torch


def write_checkpoint(folder, cfg, weights):
    """config.json + model.safetensors."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    header, blobs, at = {}, [], 0
    for name, w in weights.items():
        raw = w.contiguous().view(torch.int16).numpy().tobytes()
        header[name] = {"dtype": "BF16", "shape": list(w.shape),
                        "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    head = json.dumps(header).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)) + head + b"".join(blobs))
    return folder


def tokens_for(cfg, n, seed):
    return torch.randint(0, cfg["vocab"], (n,),
                         generator=torch.Generator().manual_seed(seed)).tolist()


class Case:
    """One configuration on disk, its weights, and remembered logits of the
    plain oracle (a module with forward(cfg, weights, tokens))."""

    def __init__(self, name, folder, cfg, weights, oracle):
        self.name = name
        self.cfg = cfg
        self.weights = weights
        self.oracle = oracle
        self.path = write_checkpoint(str(folder), cfg, weights)
        self._known = {}

    def logits(self, tokens):
        key = tuple(tokens)
        if key not in self._known:
            self._known[key] = self.oracle.forward(self.cfg, self.weights,
                                                   tokens)[0]
        return self._known[key]

    def engine(self, device, dtype, blocks=96, slots=4, **kw):
        from quoracle_amd.engine.engine import LocalEngine
        return LocalEngine([self.path], device=torch.device(device),
                           embed_model_key=None, kv_blocks_override=blocks,
                           dtype=dtype, state_slots=slots, **kw)


def error(got, want):
    """Largest per-row RMS difference, in units of the logits' RMS."""
    got, want = got.double(), want.double()
    d = (got - want).square().mean(-1).sqrt()
    return float(d.max() / want.square().mean().sqrt())


def tolerance(dtype):
    return 2e-5 if dtype == torch.float32 else 0.06


def feed(engine, path, schedule):
    """Run [[(id, tokens), ...], ...] with every place wanted; returns
    {id: logits of all its tokens so far}.  A request ends when its id is
    given as (id, None)."""
    out, live = {}, set()
    for step in schedule:
        ends = [i for i, toks in step if toks is None]
        parts = [(i, toks) for i, toks in step if toks]
        live.update(i for i, _ in parts)
        if parts:
            lg = engine.step_entries(
                path, [(i, toks, range(len(toks))) for i, toks in parts],
                live)
            at = 0
            for i, toks in parts:
                out.setdefault(i, []).append(lg[at:at + len(toks)])
                at += len(toks)
        for i in ends:
            engine.drop_session(path, i)
            live.discard(i)
    return {i: torch.cat(p) for i, p in out.items()}


def cut(tokens, sizes):
    """Split tokens into portions of the given sizes, cycling."""
    parts, at, k = [], 0, 0
    while at < len(tokens):
        n = sizes[k % len(sizes)]
        parts.append(tokens[at:at + n])
        at, k = at + n, k + 1
    return parts


def paced(parts, live, every=4):
    """Steps that feed the requests' portions {id: [tokens, ...]}, at most
    `live` of them at a time, one of every few left out of a step, each ended
    after its last portion."""
    parts = {r: list(p) for r, p in parts.items()}
    steps, waiting, now, turn = [], list(parts), [], 0
    while waiting or now:
        while waiting and len(now) < live:
            now.append(waiting.pop(0))
        step = []
        for i, r in enumerate(list(now)):
            if (turn + i) % every == every - 1 and len(now) > 1:
                continue
            step.append((r, parts[r].pop(0)))
            if not parts[r]:
                step.append((r, None))
                now.remove(r)
        steps.append(step)
        turn += 1
    return steps


def greedy(case, prompt, n, stop=257):
    """Argmax continuation by the oracle, up to the end of sequence."""
    out = []
    for _ in range(n):
        lg, _ = case.oracle.forward(case.cfg, case.weights, prompt + out)
        out.append(int(lg[-1].argmax()))
        if out[-1] == stop:
            break
    return out


def request(case, text, n, **kw):
    from quoracle_amd.engine.api import GenerateRequest
    return GenerateRequest(model_key=case.path, temperature=0.0, max_tokens=n,
                           messages=[{"role": "user", "content": text}], **kw)
