"""LocalEngine: continuous-batching inference over the HIP/CDNA4 ops.

MI355X-first design (replaces the reference's HTTP model-access layer,
reference: lib/quoracle/models/model_query.ex):

  * One LocalEngine per GPU hosts one or more models (288 GB HBM3E holds
    several 8B-class pool members comfortably).
  * Every pending agent turn across the whole spawn tree lands in one
    per-model run queue; each engine step runs ONE mixed forward per model:
    all decode sequences (1 token each) + chunked prefill tokens, exactly
    the ForwardBatch the model/kernels were designed around.
  * A sequence is unified prefill/decode: each step advances the KV cache by
    a chunk; a 1-token chunk takes the specialized decode-attention kernel.
  * Conversations are prefix-cached Sessions — consecutive consensus cycles
    of the same (agent, model) only prefill the newly appended history.
  * The engine loop runs on its own thread so host-side orchestration
    (asyncio actor runtime) overlaps GPU compute; results complete asyncio
    futures via call_soon_threadsafe.
"""

from __future__ import annotations

import asyncio
import contextlib
import os
import queue
import sys
import threading
import time
from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence, Tuple

import numpy as np
import torch

from ..models import LlamaModel, build_model, get_config
from .api import Engine, GenerateRequest, GenerateResult
from .graphs import DecodeGraphs
from .kv_cache import (BlockManager, OutOfBlocks, Session, SessionCache,
                       StateSlots)
from .sampler import FORCED, ActionGrammar, Sampler, SamplingParams
from .tokenizer import VOCAB_FLOOR, ByteTokenizer, EOS
from ..models.llama import ForwardBatch
from ..ops.hybrid import ATTN_TILE, LIN_CHUNK

BLOCK_SIZE = 16
PREFILL_CHUNK = 2048         # max prefill tokens per model per engine step
QT = 16                      # prefill tile height (must match attention.hip)
STATE_SLOTS = 64             # sequences with a recurrent state held at once

# $/1M tokens (input, output) per preset — budget plumbing needs real-ish
# numbers (reference records per-call costs: lib/quoracle/costs/recorder.ex)
_PRICES = {
    "tiny": (0.01, 0.02), "gpt2s": (0.02, 0.05),
    "llama3-8b": (0.2, 0.8), "llama3-70b": (0.9, 3.6),
    "mixtral-8x7b": (0.5, 2.0), "embed-small": (0.01, 0.01),
}


@dataclass
class _Seq:
    request: GenerateRequest
    prompt: List[int]
    session: Session
    params: SamplingParams
    grammar: Optional[ActionGrammar]
    generator: Optional[torch.Generator]
    emitted: List[int] = field(default_factory=list)
    finished: bool = False
    t_start: float = field(default_factory=time.monotonic)
    _complete: Optional[Tuple] = None        # (loop, future) | ("sync", event)
    result: Optional[GenerateResult] = None

    @property
    def known(self) -> List[int]:
        return self.prompt + self.emitted


@dataclass
class BatchEntry:
    """One sequence's part of a step: its next tokens, and the places among
    them whose logits are wanted."""
    session: Session
    tokens: List[int]
    want: Sequence[int] = ()
    seq: Optional[_Seq] = None
    error: Optional[str] = None          # set when the cache has no room


class _HostedModel:
    def __init__(self, key: str, device: torch.device, kv_blocks: int,
                 tp=None, dtype: torch.dtype = torch.bfloat16,
                 state_slots: int = STATE_SLOTS):
        self.key = key
        self.cfg = get_config(key)
        self.model = build_model(key, device, dtype=dtype, tp=tp)
        self.kv = self.model.new_kv_cache(kv_blocks, BLOCK_SIZE,
                                          state_slots=state_slots)
        self.state_slots = state_slots
        self.mgr = BlockManager(kv_blocks, BLOCK_SIZE)
        self.sessions = self._new_sessions()
        self.active: List[_Seq] = []
        self.sampler = Sampler(self.cfg.vocab_size, device)
        # each hosted model launches on its own HIP stream so pool members
        # overlap on the GPU instead of serializing through the engine loop
        self.stream = (torch.cuda.Stream(device)
                       if device.type == "cuda" else None)
        # hipGraph-captured decode step (scratch block absorbs pad-row writes)
        scratch = self.mgr.alloc(1)[0]
        maxb = min(kv_blocks, (self.cfg.max_context + BLOCK_SIZE - 1)
                   // BLOCK_SIZE)
        self.graphs = DecodeGraphs(self.model, self.kv, device, maxb, scratch)
        if tp is not None and tp.world > 1:
            # RCCL all-reduce under hipGraph capture is unvalidated on this
            # stack; TP decode stays eager until proven
            self.graphs.enabled = False

    def _new_sessions(self) -> SessionCache:
        return SessionCache(self.mgr, StateSlots(self.state_slots)
                            if self.cfg.needs_state else None)

    def stream_ctx(self):
        return (torch.cuda.stream(self.stream) if self.stream is not None
                else contextlib.nullcontext())


def _to_device(arrays: Dict[str, Sequence[int]],
               device: torch.device) -> Dict[str, torch.Tensor]:
    """int32 arrays as views of one buffer: a single host-to-device copy."""
    host = {k: np.asarray(v, dtype=np.int32) for k, v in arrays.items()}
    flat = torch.from_numpy(
        np.concatenate([a.ravel() for a in host.values()])).to(device)
    out, at = {}, 0
    for k, a in host.items():
        out[k] = flat[at:at + a.size].view(a.shape)
        at += a.size
    return out


class LocalEngine(Engine):
    def __init__(self, model_keys: Sequence[str],
                 device: Optional[torch.device] = None,
                 kv_gb_per_model: float = 4.0,
                 embed_model_key: Optional[str] = "embed-small",
                 kv_blocks_override: Optional[int] = None,
                 prefill_chunk: int = PREFILL_CHUNK,
                 tp=None, dtype: torch.dtype = torch.bfloat16,
                 state_slots: int = STATE_SLOTS):
        self.device = device or torch.device(
            "cuda:0" if torch.cuda.is_available() else "cpu")
        self.tokenizer = ByteTokenizer()
        self.prefill_chunk = prefill_chunk
        self.models: Dict[str, _HostedModel] = {}
        for key in model_keys:
            cfg = get_config(key)
            if kv_blocks_override is not None:
                blocks = kv_blocks_override
            else:
                per_block = max(1, cfg.kv_bytes_per_token(dtype.itemsize)
                                * BLOCK_SIZE)
                blocks = max(8, int(kv_gb_per_model * (1 << 30) / per_block))
                # small models would otherwise allocate millions of blocks
                # for the same byte budget; 2M tokens of KV is plenty
                blocks = min(blocks, (2 << 20) // BLOCK_SIZE)
            self.models[key] = _HostedModel(
                key, self.device, blocks, tp=tp, dtype=dtype,
                state_slots=state_slots)
        self.embed_model: Optional[LlamaModel] = None
        if embed_model_key:
            self.embed_model = LlamaModel(embed_model_key, self.device)
        self._inbox: "queue.Queue[_Seq]" = queue.Queue()
        self._gpu_lock = threading.Lock()
        self._thread: Optional[threading.Thread] = None
        self._running = False
        self._wake = threading.Event()
        # telemetry (read by bench/monitor; written only by the engine thread)
        self.stats = {"engine_steps": 0, "forward_tokens": 0,
                      "decode_tokens": 0, "prefill_tokens": 0,
                      "requests_done": 0, "prefix_hit_tokens": 0}
        self._log_every = int(os.environ.get("QUORACLE_ENGINE_LOG", "0"))
        self._roctx = bool(os.environ.get("QUORACLE_ROCTX"))
        # QUORACLE_CHECK=1: synchronize after every launch phase so async
        # HIP faults surface at their source (SURVEY.md §5.2 debug mode)
        self._strict_sync = bool(os.environ.get("QUORACLE_CHECK"))

    # -- lifecycle -----------------------------------------------------------

    def start(self) -> "LocalEngine":
        if self._thread is None:
            if self.device.type == "cuda":
                torch.cuda.synchronize(self.device)   # weight init done
                self.precapture_graphs()
            self._running = True
            self._thread = threading.Thread(target=self._loop, daemon=True,
                                            name="quoracle-engine")
            self._thread.start()
        return self

    def precapture_graphs(self, buckets=(1, 2, 4, 8, 16)) -> None:
        """hipGraph-capture each model's decode step per batch bucket while
        the GPU is quiescent; decode steps then replay instead of
        relaunching ~260 kernels eagerly."""
        t0 = time.monotonic()
        for hm in self.models.values():
            hm.graphs.precapture(buckets)
        if self.device.type == "cuda":
            torch.cuda.synchronize(self.device)
            print(f"[engine] graph precapture done in "
                  f"{time.monotonic() - t0:.1f}s "
                  f"({sum(len(h.graphs.graphs) for h in self.models.values())}"
                  f" graphs)", file=sys.stderr, flush=True)

    def stop(self) -> None:
        self._running = False
        self._wake.set()
        if self._thread:
            self._thread.join(timeout=30)
            self._thread = None

    # -- Engine protocol -----------------------------------------------------

    async def generate(self, request: GenerateRequest) -> GenerateResult:
        loop = asyncio.get_running_loop()
        fut: asyncio.Future = loop.create_future()
        err = self._submit(request, ("async", loop, fut))
        if err is not None:
            return err
        return await fut

    def generate_sync(self, request: GenerateRequest,
                      timeout: Optional[float] = None) -> GenerateResult:
        """Blocking path for tests / non-async callers; drives the engine
        inline when the loop thread is not running."""
        ev = threading.Event()
        box: List[GenerateResult] = []
        err = self._submit(request, ("sync", ev, box))
        if err is not None:
            return err
        if self._thread is None:
            deadline = None if timeout is None else time.monotonic() + timeout
            while not ev.is_set():
                self.step()
                if deadline and time.monotonic() > deadline:
                    raise TimeoutError("generate_sync timed out")
        else:
            ev.wait(timeout)
        if not box:
            raise TimeoutError("generate_sync timed out")
        return box[0]

    async def embed(self, texts: List[str]) -> Sequence[Sequence[float]]:
        return await asyncio.get_running_loop().run_in_executor(
            None, self.embed_sync, list(texts))

    def embed_sync(self, texts: List[str]) -> Sequence[Sequence[float]]:
        if self.embed_model is None:
            raise RuntimeError("no embedding model hosted")
        batches = []
        for t in texts:
            ids = self.tokenizer.encode(t)[:512] or [EOS]
            batches.append(torch.tensor(ids, dtype=torch.int32,
                                        device=self.device))
        with self._gpu_lock:
            hid = self.embed_model.embed_texts_hidden(batches)
        norm = hid.norm(dim=-1, keepdim=True).clamp_min(1e-8)
        return (hid / norm).cpu().tolist()

    def similarity_matrix(self, texts: List[str]):
        """Pairwise cosine matrix of the texts' embeddings — embedding
        forward + the fused cosine_sim_matrix kernel in one GPU pass
        (the consensus vote's hot path)."""
        if self.embed_model is None:
            raise RuntimeError("no embedding model hosted")
        batches = []
        for t in texts:
            ids_ = self.tokenizer.encode(t)[:512] or [EOS]
            batches.append(torch.tensor(ids_, dtype=torch.int32,
                                        device=self.device))
        from ..ops import dispatch as D
        with self._gpu_lock:
            hid = self.embed_model.embed_texts_hidden(batches).float()
            out = torch.empty((hid.shape[0], hid.shape[0]),
                              dtype=torch.float32, device=hid.device)
            D.cosine_sim_matrix(out, hid)
        return out.cpu().tolist()

    def count_tokens(self, text: str) -> int:
        return self.tokenizer.count(text)

    def context_limit(self, model_key: str) -> int:
        return get_config(model_key).max_context

    def output_limit(self, model_key: str) -> int:
        return get_config(model_key).max_output

    def drop_session(self, model_key: str, session_id: str) -> None:
        hm = self.models.get(model_key)
        if hm:
            hm.sessions.drop(session_id)

    # -- request intake ------------------------------------------------------

    def _submit(self, request: GenerateRequest, completion,
                enqueue: bool = True) -> Optional[GenerateResult]:
        hm = self.models.get(request.model_key)
        if hm is None:
            return GenerateResult(model_key=request.model_key,
                                  error=f"model_not_hosted:{request.model_key}")
        if hm.cfg.vocab_size < VOCAB_FLOOR:
            return GenerateResult(
                model_key=request.model_key,
                error=f"vocabulary_too_small:{hm.cfg.vocab_size}")
        prompt = self.tokenizer.render_messages(request.messages)
        if len(prompt) > hm.cfg.max_context:
            return GenerateResult(model_key=request.model_key,
                                  error="context_overflow",
                                  input_tokens=len(prompt))
        max_tokens = min(request.max_tokens, hm.cfg.max_output,
                         hm.cfg.max_context - len(prompt))
        if request.action_grammar:
            # the grammar terminates by itself (~600 tokens worst case);
            # never truncate it into unparseable JSON — but stay inside the
            # model's remaining window or positions run past max_context
            max_tokens = min(max(max_tokens, 1024),
                             hm.cfg.max_context - len(prompt))
        params = SamplingParams(
            temperature=request.temperature, top_p=request.top_p,
            max_tokens=max_tokens, seed=request.seed)
        grammar = None
        if request.action_grammar:
            grammar = ActionGrammar(
                request.allowed_actions
                or ["orient", "send_message", "todo", "wait"],
                context=request.grammar_context)
        gen = None
        if request.seed is not None:
            gen = torch.Generator(device=self.device)
            gen.manual_seed(request.seed)
        sid = request.session_id or f"anon-{id(request)}"
        seq = _Seq(request=request, prompt=prompt, session=None,  # type: ignore
                   params=params, grammar=grammar, generator=gen,
                   _complete=completion)
        seq._session_id = sid                                     # type: ignore
        if not enqueue:
            self._made_seq = seq
            return None
        self._inbox.put(seq)
        self._wake.set()
        return None

    # -- engine loop ---------------------------------------------------------

    def _loop(self) -> None:
        while self._running:
            worked = self.step()
            if not worked:
                self._wake.wait(timeout=0.005)
                self._wake.clear()

    def step(self) -> bool:
        """One engine step: admit new work, then for every model with pending
        sequences LAUNCH one mixed forward on that model's own stream (phase
        1, async) and only then sample (phase 2, syncs per stream) — pool
        members overlap on the GPU.  Returns True if any work was done."""
        self._admit()
        pending = []
        for hm in self.models.values():
            if not hm.active:
                continue
            try:
                with self._gpu_lock:
                    ctxt = self._launch_model(hm)
            except Exception as exc:  # noqa: BLE001 — fail loud, not hang
                self._crash_model(hm, exc)
                continue
            if ctxt is not None:
                if self._strict_sync and self.device.type == "cuda":
                    torch.cuda.synchronize(self.device)
                pending.append((hm, ctxt))
        for hm, ctxt in pending:
            try:
                with self._gpu_lock:
                    self._sample_model(hm, *ctxt)
            except Exception as exc:  # noqa: BLE001
                self._crash_model(hm, exc)
        return bool(pending)

    def _crash_model(self, hm: _HostedModel, exc: Exception) -> None:
        import traceback
        traceback.print_exc()
        print(f"[engine {hm.key}] step failed: {exc}; failing "
              f"{len(hm.active)} in-flight requests",
              file=sys.stderr, flush=True)
        crashed = list(hm.active)
        for seq in crashed:
            seq.result = GenerateResult(
                model_key=hm.key, error=f"engine_error:{exc}")
        self._finish(hm, crashed)
        # the failed step may have recorded tokens whose K/V or recurrent
        # state was never written
        for seq in crashed:
            if seq.session is not None:
                hm.sessions.drop(seq.session.session_id)
        # Watchdog: repeated failures mean corrupted
        # device state — rebuild the model's KV world.  Conversation
        # history lives in the orchestrator, so sessions re-prefill
        # lazily via the prefix cache on the next request; the failed
        # shard simply drops out of votes until then (consensus already
        # tolerates partial pools).
        hm.crash_count = getattr(hm, "crash_count", 0) + 1
        if hm.crash_count >= 2:
            self.reset_model(hm.key)

    def reset_model(self, key: str) -> None:
        """Rebuild a hosted model's KV cache, block manager and sessions
        after a device fault; weights stay resident (they are immutable)."""
        hm = self.models.get(key)
        if hm is None:
            return
        print(f"[engine {key}] watchdog reset: rebuilding KV state",
              file=sys.stderr, flush=True)
        crashed = list(hm.active)
        for seq in crashed:
            if seq.result is None:
                seq.result = GenerateResult(model_key=key,
                                            error="engine_reset")
        self._finish(hm, crashed)
        blocks = hm.mgr.num_blocks
        bs = hm.kv.block_size
        hm.kv.clear()
        hm.mgr = BlockManager(blocks, bs)
        hm.sessions = hm._new_sessions()
        scratch = hm.mgr.alloc(1)[0]
        hm.graphs.scratch_block = scratch
        hm.crash_count = 0

    def _admit(self) -> None:
        if getattr(self, "_tp_direct", False):
            return      # lockstep engines admit via the admit-broadcast only
        while True:
            try:
                seq = self._inbox.get_nowait()
            except queue.Empty:
                return
            self._admit_seq(seq)

    def _admit_seq(self, seq: "_Seq") -> None:
        hm = self.models[seq.request.model_key]
        sess = hm.sessions.get_or_create(seq._session_id)   # type: ignore
        hit = hm.sessions.match_prefix(sess, seq.prompt)
        self.stats["prefix_hit_tokens"] += hit
        seq.session = sess
        hm.active.append(seq)

    def _expand_forced(self, hm: _HostedModel, seq: _Seq) -> None:
        """Append the grammar's next run of FORCED tokens in one go: known
        structural JSON needs no per-token decode — the run becomes a
        chunked prefill, collapsing ~60% of generated tokens into a handful
        of forwards."""
        g = seq.grammar
        if g is None or seq.finished:
            return
        while not seq.finished and not g.done and g.current()[0] == FORCED:
            tok = g.advance(0)
            seq.emitted.append(tok)
            if (tok == EOS or g.done
                    or len(seq.emitted) >= seq.params.max_tokens):
                seq.finished = True
                seq.result = self._make_result(hm, seq)
                self.stats["requests_done"] += 1

    def _launch_model(self, hm: _HostedModel):
        """Schedule one step of a model's sequences and run it as one batch.
        Returns what _sample_model takes, or None when there is nothing."""
        entries: List[BatchEntry] = []
        early_done: List[_Seq] = []
        budget = self.prefill_chunk
        active_ids = [s.session.session_id for s in hm.active]
        for seq in hm.active:
            self._expand_forced(hm, seq)
            if seq.finished:
                early_done.append(seq)
                continue
            cached = len(seq.session.token_ids)
            remaining = len(seq.known) - cached
            n = 1 if remaining <= 1 else min(remaining, budget)
            if n <= 0:
                continue
            if not hm.sessions.place(seq.session, active_ids):
                continue       # every state slot is held: wait for one
            if n > 1 or remaining > 1:
                budget -= n
            entries.append(BatchEntry(
                seq.session, seq.known[cached:cached + n],
                want=(n - 1,) if n == remaining else (), seq=seq))

        if early_done:
            self._finish(hm, early_done)
        if not entries:
            return None
        rows, logits, on_default = self.run_batch(hm, entries, active_ids)
        failed = []
        for e in entries:
            if e.error is not None:
                e.seq.result = GenerateResult(model_key=hm.key, error=e.error)
                failed.append(e.seq)
        if rows is None:
            self._finish(hm, failed)
            return None
        return ([e.seq for e, _ in rows], logits, failed, on_default)

    def run_batch(self, hm: _HostedModel, entries: Sequence[BatchEntry],
                  active_ids: Sequence[str]):
        """Run the entries as ONE mixed batch over the model's cache: single
        tokens as decode rows, longer runs as prefill rows.

        Returns (rows, logits, on_default_stream): rows lists (entry, place)
        of each logits row; rows is None when no entry found room (their
        `error` is set), logits None when none are wanted."""
        for e in entries:
            end = len(e.session.token_ids) + len(e.tokens)
            if not e.tokens or end > hm.cfg.max_context:
                raise ValueError(
                    f"{len(e.tokens)} tokens up to position {end} of "
                    f"{hm.cfg.max_context}")
            if min(e.tokens) < 0 or max(e.tokens) >= hm.cfg.vocab_size:
                raise ValueError(f"token outside 0..{hm.cfg.vocab_size - 1}")
            if any(not 0 <= w < len(e.tokens) for w in e.want):
                raise ValueError("logits wanted outside the entry's tokens")

        starts: List[int] = []
        slots: List[int] = []
        placed: List[BatchEntry] = []
        # single tokens first, then portions; where the model treats short
        # portions differently, those before the long ones
        split = getattr(hm.model, "expand_from", None) or 2
        for e in sorted(entries, key=lambda e: (len(e.tokens) > 1)
                        + (len(e.tokens) >= split)):
            start = len(e.session.token_ids)
            try:
                slots.extend(hm.sessions.extend(e.session, e.tokens,
                                                active=active_ids))
            except OutOfBlocks as exc:
                e.error = f"kv_exhausted:{exc}"
                continue
            starts.append(start)
            placed.append(e)
        if not placed:
            return None, None, False
        n_decode = sum(1 for e in placed if len(e.tokens) == 1)

        # pure-decode steps replay the hipGraph-captured step when possible.
        # Replay + its input copies run on the DEFAULT stream: hipGraph
        # replay launched from a side stream deadlocks on ROCm 7.2 (observed
        # on MI355X; graph kernels never complete), so graph steps serialize
        # across models while eager prefill keeps per-model streams.
        if n_decode == len(placed):
            if hm.stream is not None:
                # order after this model's eager (prefill) stream, and make
                # that stream wait for the replay before later prefills
                torch.cuda.current_stream(self.device).wait_stream(hm.stream)
            logits = hm.graphs.run(
                [e.tokens[0] for e in placed], starts, slots,
                [e.session.blocks for e in placed], [s + 1 for s in starts],
                # the full block tuple participates in the staging key:
                # after eviction + re-prefill a session can reuse the same
                # length and tail block with different middle blocks
                bt_keys=[(e.session.session_id,
                          hash(tuple(e.session.blocks))) for e in placed],
                state_slots=[e.session.state_slot for e in placed])
            if logits is not None:
                if hm.stream is not None:
                    hm.stream.wait_stream(
                        torch.cuda.current_stream(self.device))
                st = self.stats
                st["engine_steps"] += 1
                st["graph_steps"] = st.get("graph_steps", 0) + 1
                st["forward_tokens"] += n_decode
                st["decode_tokens"] += n_decode
                keep = [i for i, e in enumerate(placed) if len(e.want)]
                if not keep:
                    return [], None, True
                if len(keep) < len(placed):
                    logits = logits[keep]
                return [(placed[i], 0) for i in keep], logits, True
        return self._run_eager(hm, placed, starts, slots, n_decode)

    def _run_eager(self, hm: _HostedModel, placed: List[BatchEntry],
                   starts: List[int], slots: List[int], n_decode: int):
        dev = self.device
        tokens: List[int] = []
        positions: List[int] = []
        rows: List[Tuple[BatchEntry, int]] = []
        sample_rows: List[int] = []
        # 128-row tiles match the default T12 prefill kernel (352 TF);
        # QUORACLE_MFMA64/QUORACLE_MFMA32 fall back (Llama family)
        if hm.cfg.is_hybrid:
            big_step = ATTN_TILE
        elif os.environ.get("QUORACLE_MFMA32"):
            big_step = 32
        elif os.environ.get("QUORACLE_MFMA64"):
            big_step = 64
        else:
            big_step = 128
        tiles: Dict[str, List[int]] = {
            f"{t}_{f}": [] for t in ("tile", "tile32")
            for f in ("q0", "qn", "seq", "pos0")}
        row_seq: List[int] = []
        seg: Dict[str, List[int]] = {"row0": [], "len": [], "chunk0": [0]}
        chunk: Dict[str, List[int]] = {"row0": [], "len": []}
        max_kv = 0
        # portions this long attend over keys and values made from the cached
        # latents of their whole context; shorter ones take 16-row tiles
        split = getattr(hm.model, "expand_from", None)
        ctx_slots: List[np.ndarray] = []
        ctx0: List[int] = []
        n_ctx, n_latent = 0, n_decode
        for i, (e, start) in enumerate(zip(placed, starts)):
            row, n = len(tokens), len(e.tokens)
            tokens.extend(e.tokens)
            positions.extend(range(start, start + n))
            for w in e.want:
                rows.append((e, w))
                sample_rows.append(row + w)
            row_seq.extend([i] * n)
            if i < n_decode:
                continue
            max_kv = max(max_kv, start + n)
            if not hm.cfg.is_hybrid:
                kinds = (("tile", QT), ("tile32", big_step))
            elif split is not None and n < split:
                kinds = (("tile", QT),)
                n_latent = row + n
            else:
                kinds = (("tile32", big_step),)
            for name, step in kinds:
                for off in range(0, n, step):
                    tiles[name + "_q0"].append(row + off)
                    tiles[name + "_qn"].append(min(step, n - off))
                    tiles[name + "_seq"].append(i)
                    tiles[name + "_pos0"].append(start + off)
            if split is not None and n >= split:
                at = np.arange(start + n)
                blocks = np.asarray(e.session.blocks, dtype=np.int32)
                ctx_slots.append(blocks[at // BLOCK_SIZE] * BLOCK_SIZE
                                 + at % BLOCK_SIZE)
                ctx0 += [n_ctx] * -(-n // big_step)
                n_ctx += start + n
            seg["row0"].append(row)
            seg["len"].append(n)
            for off in range(0, n, LIN_CHUNK):
                chunk["row0"].append(row + off)
                chunk["len"].append(min(LIN_CHUNK, n - off))
            seg["chunk0"].append(len(chunk["row0"]))

        maxb = max(len(e.session.blocks) for e in placed)
        # numpy staging: per-row torch.tensor() creation measured ~20us
        # each on the eager step path
        bt_np = np.zeros((len(placed), maxb), dtype=np.int32)
        for i, e in enumerate(placed):
            bt_np[i, :len(e.session.blocks)] = e.session.blocks
        arrays = {"tokens": tokens, "positions": positions, "slots": slots,
                  "block_tables": bt_np, **tiles}
        if n_decode:
            arrays["ctx_lens"] = [s + 1 for s in starts[:n_decode]]
        if hm.cfg.is_hybrid:
            arrays["row_seq"] = row_seq
        if hm.cfg.needs_state:
            arrays.update(
                seg_row0=seg["row0"], seg_len=seg["len"],
                seg_chunk0=seg["chunk0"], chunk_row0=chunk["row0"],
                chunk_len=chunk["len"],
                state_slots=[e.session.state_slot for e in placed])
        if ctx_slots:
            arrays["ctx_slots"] = np.concatenate(ctx_slots)
            arrays["tile32_ctx0"] = ctx0

        t_fwd = time.monotonic()
        # rocprof/omnitrace attribution: roctx ranges around each eager
        # forward; QUORACLE_ROCTX=1 enables
        if self._roctx:
            torch.cuda.nvtx.range_push(
                f"fwd:{hm.key}:T{len(tokens)}:d{n_decode}")
        # batch tensors are one H2D copy: made on the model's stream so the
        # forward (same stream) is ordered after it without a sync
        with hm.stream_ctx():
            batch = ForwardBatch(
                n_decode=n_decode, max_ctx=max(starts[:n_decode], default=-1)
                + 1, max_kv=max_kv, n_latent=n_latent,
                **_to_device(arrays, dev))
            hidden = hm.model.forward(batch, hm.kv)
            logits = None
            if sample_rows:
                at = torch.tensor(sample_rows, dtype=torch.long, device=dev)
                logits = hm.model.compute_logits(hidden, at)
        if self._roctx:
            torch.cuda.nvtx.range_pop()
        st = self.stats
        st["engine_steps"] += 1
        st["forward_tokens"] += len(tokens)
        st["decode_tokens"] += n_decode
        st["prefill_tokens"] += len(tokens) - n_decode
        if self._log_every and st["engine_steps"] % self._log_every == 0:
            print(f"[engine {hm.key}] step={st['engine_steps']} "
                  f"T={len(tokens)} dec={n_decode} active={len(hm.active)} "
                  f"launch_ms={(time.monotonic() - t_fwd) * 1e3:.1f}",
                  file=sys.stderr, flush=True)
        return rows, logits, False

    # -- direct stepping -----------------------------------------------------

    def step_entries(self, model_key: str,
                     entries: Sequence[Tuple[str, Sequence[int],
                                             Sequence[int]]],
                     live: Sequence[str] = ()) -> Optional[torch.Tensor]:
        """Feed given tokens instead of sampled ones: each entry is (session
        id, next tokens, places wanted), all of them one batch of the same
        step that generation runs.  Sessions named here or in `live` are not
        evicted.  Returns the wanted logits in the order of the entries and
        of their places, [wanted, vocab] float32 on the CPU."""
        hm = self.models[model_key]
        batch = [BatchEntry(hm.sessions.get_or_create(sid), list(tokens),
                            want=tuple(want)) for sid, tokens, want in entries]
        keep = set(live) | {e.session.session_id for e in batch}
        with self._gpu_lock:
            rows, logits, on_default = self.run_batch(hm, batch, list(keep))
            for e in batch:
                if e.error is not None:
                    raise OutOfBlocks(e.error)
            if not rows:
                return None
            with (contextlib.nullcontext() if on_default
                  else hm.stream_ctx()):
                out = logits.cpu()
        at = {(id(e), w): i for i, (e, w) in enumerate(rows)}
        return out[[at[id(e), w] for e in batch for w in e.want]]

    def _sample_model(self, hm: _HostedModel, sample_seqs, logits,
                      failed, on_default_stream=False) -> None:
        done: List[_Seq] = list(failed)
        if logits is not None:
            with (contextlib.nullcontext() if on_default_stream
                  else hm.stream_ctx()):
                ids = hm.sampler.sample(
                    logits, [s.params for s in sample_seqs],
                    [s.grammar for s in sample_seqs],
                    [s.generator for s in sample_seqs])
            for seq, tok in zip(sample_seqs, ids):
                seq.emitted.append(tok)
                if (tok == EOS or len(seq.emitted) >= seq.params.max_tokens
                        or (seq.grammar is not None and seq.grammar.done)):
                    seq.finished = True
                    seq.result = self._make_result(hm, seq)
                    self.stats["requests_done"] += 1
                    done.append(seq)
        self._finish(hm, done)

    def _make_result(self, hm: _HostedModel, seq: _Seq) -> GenerateResult:
        out_ids = [t for t in seq.emitted if t != EOS]
        text = self.tokenizer.decode(out_ids)
        n_in, n_out = len(seq.prompt), len(seq.emitted)
        pin, pout = _PRICES.get(hm.cfg.name, (0.1, 0.4))
        return GenerateResult(
            model_key=hm.key, text=text, input_tokens=n_in,
            output_tokens=n_out,
            latency_ms=(time.monotonic() - seq.t_start) * 1e3,
            cost=(n_in * pin + n_out * pout) / 1e6)

    def _finish(self, hm: _HostedModel, done: List[_Seq]) -> None:
        for seq in done:
            if seq in hm.active:
                hm.active.remove(seq)
            # one-shot (anonymous) sessions release their KV immediately;
            # named sessions persist for prefix reuse
            if not seq.request.session_id and seq.session is not None:
                hm.sessions.drop(seq.session.session_id)
            comp = seq._complete
            if comp is None:
                continue
            if comp[0] == "async":
                _, loop, fut = comp
                loop.call_soon_threadsafe(
                    lambda f=fut, r=seq.result: f.done() or f.set_result(r))
            elif comp[0] == "cb":
                comp[1](seq.result)
            else:
                _, ev, box = comp
                box.append(seq.result)
                ev.set()
