"""Koridra through the engine against the plain oracle: whole prompts,
token-by-token decoding, portions, mixed batches, reused pages and slots, and
generation by the scheduler.  The same tests run on the CPU (plain ops) and,
marked gpu, on the HIP kernels in float32 and bf16."""

import json
import os
import subprocess
import sys

import pytest
import torch

import koridra_oracle as oracle
from hybrid_cases import (cut, error, feed, greedy, paced, request, tokens_for,
                          tolerance)
from koridra_cases import CONFIGS, Case

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
WHERE = [
    pytest.param(("cpu", torch.float32), id="cpu"),
    pytest.param(("cuda:0", torch.float32), id="gpu-f32",
                 marks=pytest.mark.gpu),
    pytest.param(("cuda:0", torch.bfloat16), id="gpu-bf16",
                 marks=pytest.mark.gpu),
]


@pytest.fixture(scope="module")
def cases(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            made[name] = Case(name, tmp_path_factory.mktemp(name))
        return made[name]
    return get


def check(case, got, requests, dtype):
    for rid, toks in requests.items():
        err = error(got[rid], case.logits(toks))
        assert err < tolerance(dtype), f"{case.name} {rid}: {err:.2e}"


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("where", WHERE)
def test_whole_prompts(cases, name, where):
    case = cases(name)
    eng = case.engine(*where)
    # one token, a few, across page/tile/chunk borders
    reqs = {f"r{n}": tokens_for(case.cfg, n, n) for n in (1, 2, 65, 150)}
    got = {}
    for rid, toks in reqs.items():
        got.update(feed(eng, case.path, [[(rid, toks)], [(rid, None)]]))
    check(case, got, reqs, where[1])


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("where", WHERE)
def test_decoding_equals_prefill(cases, name, where):
    """Every token from the first one alone, and after a prompt."""
    case = cases(name)
    toks = tokens_for(case.cfg, 150, 150)
    for head in (0, 70):
        eng = case.engine(*where)
        eng.precapture_graphs((1, 2))
        steps = ([[("a", toks[:head])]] if head else []) \
            + [[("a", [t])] for t in toks[head:]]
        check(case, feed(eng, case.path, steps), {"a": toks}, where[1])


@pytest.mark.parametrize("sizes", [[2], [3, 2, 17], [64, 1, 63], [37, 36, 1]],
                         ids=str)
@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("where", WHERE)
def test_portions(cases, name, where, sizes):
    case = cases(name)
    toks = tokens_for(case.cfg, 150, 150)
    eng = case.engine(*where)
    got = feed(eng, case.path, [[("a", p)] for p in cut(toks, sizes)])
    check(case, got, {"a": toks}, where[1])


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("where", WHERE)
def test_mixed_batches_and_reuse(cases, name, where):
    """Unequal requests side by side, some decoding, some in portions, one
    paused; then new ones in the pages and slots that were given back, with a
    pool that does not hold all of them at once."""
    case = cases(name)
    lens = {"a": 90, "b": 33, "c": 5, "d": 110, "e": 64, "f": 90}
    reqs = {r: tokens_for(case.cfg, n, 7 * n + i)
            for i, (r, n) in enumerate(lens.items())}
    parts = {"a": cut(reqs["a"], [20, 1, 1, 9]), "b": cut(reqs["b"], [2, 1]),
             "c": cut(reqs["c"], [1]), "d": cut(reqs["d"], [50, 3, 1]),
             "e": cut(reqs["e"], [16]), "f": cut(reqs["f"], [1, 31])}
    eng = case.engine(*where, blocks=20, slots=3)
    eng.precapture_graphs((1, 2, 4))
    got = feed(eng, case.path, paced(parts, 3))
    check(case, got, reqs, where[1])
    hm = eng.models[case.path]
    assert hm.mgr.free_blocks == 19 and hm.sessions.states.free_slots == 3


@pytest.mark.parametrize("where", WHERE)
def test_batch_does_not_matter(cases, where):
    """The same request alone and beside others: equal up to rounding."""
    case = cases("tiles")
    toks, other = tokens_for(case.cfg, 60, 1), tokens_for(case.cfg, 90, 2)
    alone = feed(case.engine(*where), case.path,
                 [[("a", toks[:41])], [("a", toks[41:])]])["a"]
    eng = case.engine(*where)
    eng.models[case.path].mgr.alloc(5)       # other pages than before
    both = feed(eng, case.path,
                [[("b", other[:10])], [("b", other[10:30]), ("a", toks[:41])],
                 [("a", toks[41:]), ("b", other[30:])]])["a"]
    assert error(both, alone) < tolerance(where[1]) / 2


@pytest.mark.parametrize("where", WHERE)
def test_long_decoding(cases, where):
    case = cases("tiles")
    toks = tokens_for(case.cfg, 420, 4)
    eng = case.engine(*where)
    eng.precapture_graphs((1,))
    got = feed(eng, case.path, [[("a", toks[:40])]]
               + [[("a", [t])] for t in toks[40:]])["a"]
    want = case.logits(toks)
    assert error(got, want) < tolerance(where[1])
    # no drift: the last part is as good as the whole
    assert error(got[-50:], want[-50:]) < tolerance(where[1])


# -- the oracle notices what it should ---------------------------------------

def _bent(mechanism):
    """Oracle logits with one mechanism bent."""
    saved = {k: getattr(oracle, k) for k in
             ("sees", "sink_attention", "decayed_recurrence",
              "rotary_frequencies")}
    cfg = json.loads(json.dumps(CONFIGS["tiles"]))
    if mechanism == "chunk off by one":
        oracle.sees = lambda i, j, c: saved["sees"](i + 1, j + 1, c)
    elif mechanism == "no chunk":
        oracle.sees = lambda i, j, c: j <= i
    elif mechanism == "no sink":
        def plain(q, k, v, scale, chunk, positions=None):
            o = saved["sink_attention"](q, k, v, scale, chunk, positions)
            ones = saved["sink_attention"](q, k, torch.ones_like(v), scale,
                                           chunk, positions)
            return o / ones
        oracle.sink_attention = plain
    elif mechanism == "lost state":
        def lossy(q, k, v, decay, state=None):
            a, s = saved["decayed_recurrence"](q[:64], k[:64], v[:64],
                                               decay[:64])
            b, _ = saved["decayed_recurrence"](q[64:], k[64:], v[64:],
                                               decay[64:] if decay.shape[0] > 1
                                               else decay, s * 0.97)
            return torch.cat([a, b]), s
        oracle.decayed_recurrence = lossy
    elif mechanism == "no scaling":
        def unscaled(rot):
            return saved["rotary_frequencies"](
                {"dims": rot["dims"], "base": rot["base"]})
        oracle.rotary_frequencies = unscaled
    return cfg, saved


@pytest.mark.parametrize("mechanism", ["chunk off by one", "no chunk",
                                       "no sink", "lost state", "no scaling"])
def test_oracle_shows_a_wrong_mechanism(cases, mechanism):
    """A small mistake moves the logits by far more than the tolerance, so
    the comparisons above would show it."""
    case = cases("tiles")
    toks = tokens_for(case.cfg, 100, 9)
    right = case.logits(toks)
    cfg, saved = _bent(mechanism)
    try:
        wrong = oracle.forward(cfg, case.weights, toks)[0]
    finally:
        for k, f in saved.items():
            setattr(oracle, k, f)
    assert error(wrong, right) > 20 * tolerance(torch.float32)


# -- generation --------------------------------------------------------------

@pytest.mark.parametrize("where", WHERE[:2])
@pytest.mark.parametrize("chunk", [2048, 7])
def test_greedy_generation(cases, where, chunk):
    """Through generate_sync and the scheduler, prompts prefilled whole or in
    portions of 7, against argmax of the oracle."""
    case = cases("tiles")
    eng = case.engine(*where, prefill_chunk=chunk)
    prompt = eng.tokenizer.render_messages(
        [{"role": "user", "content": "a chunk border lies in this"}])
    want = greedy(case, prompt, 12)
    r = eng.generate_sync(request(case, "a chunk border lies in this", 12),
                          timeout=120)
    assert r.ok, r.error
    assert r.output_tokens == len(want)
    assert r.text == eng.tokenizer.decode([t for t in want if t != 257])


@pytest.mark.parametrize("where", WHERE[:2])
def test_more_requests_than_slots(cases, where):
    """Five requests share two state slots: three wait, all come out as they
    do alone, and everything is given back."""
    case = cases("odd")
    texts = ["one", "number two", "3", "the fourth request", "v"]
    alone = {}
    for t in texts:
        alone[t] = case.engine(*where).generate_sync(
            request(case, t, 9), timeout=120).text
    eng = case.engine(*where, slots=2)
    done = {}
    for t in texts:
        eng._submit(request(case, t, 9),
                    ("cb", lambda r, t=t: done.__setitem__(t, r)))
    for _ in range(400):
        if len(done) == len(texts):
            break
        eng.step()
    assert {t: r.text for t, r in done.items()} == alone
    hm = eng.models[case.path]
    assert hm.sessions.states.free_slots == 2 and not hm.active


@pytest.mark.parametrize("where", WHERE[:2])
def test_session_continues_or_starts_over(cases, where):
    """A prompt that continues a cached session reuses its state; one that
    leaves it starts from nothing.  Either way the text is the same as in a
    fresh engine."""
    case = cases("odd")
    eng = case.engine(*where)
    first = eng.generate_sync(request(case, "hello", 6, session_id="s"),
                              timeout=120)
    sess = eng.models[case.path].sessions.get_or_create("s")
    held = list(sess.token_ids)
    # same prompt again: its state has moved past the prompt, so start over
    again = eng.generate_sync(request(case, "hello", 6, session_id="s"),
                              timeout=120)
    assert again.text == first.text
    assert eng.stats["prefix_hit_tokens"] == 0
    # a prompt that contains everything cached so far
    sid = eng.models[case.path].sessions
    assert sid.match_prefix(sess, held + [1, 2]) == len(held)
    # another text in the same session
    other = eng.generate_sync(request(case, "help", 6, session_id="s"),
                              timeout=120)
    fresh = case.engine(*where).generate_sync(request(case, "help", 6),
                                              timeout=120)
    assert other.text == fresh.text


def test_idle_sessions_make_room(cases):
    """Named sessions keep their slot when idle and lose it to new work."""
    case = cases("odd")
    eng = case.engine("cpu", torch.float32, slots=1)
    for name in ("x", "y", "x"):
        r = eng.generate_sync(request(case, name, 3, session_id=name),
                              timeout=60)
        assert r.ok, r.error


def test_bad_input_is_refused(cases):
    case = cases("odd")
    eng = case.engine("cpu", torch.float32, blocks=60)
    with pytest.raises(ValueError):
        eng.step_entries(case.path, [("a", [case.cfg["vocab"]], [])])
    with pytest.raises(ValueError):
        eng.step_entries(case.path, [("a", [-1], [])])
    with pytest.raises(ValueError):          # past the position table
        eng.step_entries(
            case.path,
            [("a", [1] * (case.cfg["max_positions"] + 1), [])])
    with pytest.raises(ValueError):
        eng.step_entries(case.path, [("a", [1], [1])])


def test_failed_step_drops_its_sessions(cases, monkeypatch):
    """After a step that raised, neither K/V nor state of its sessions may be
    trusted: the next request of the session starts over."""
    case = cases("odd")
    eng = case.engine("cpu", torch.float32)
    want = eng.generate_sync(request(case, "abc", 4), timeout=60).text
    hm = eng.models[case.path]
    good = hm.model.forward
    monkeypatch.setattr(hm.model, "forward",
                        lambda *a, **k: (_ for _ in ()).throw(
                            RuntimeError("planted")))
    r = eng.generate_sync(request(case, "abc", 4, session_id="s"),
                          timeout=60)
    assert not r.ok
    monkeypatch.setattr(hm.model, "forward", good)
    r = eng.generate_sync(request(case, "abc", 4, session_id="s"),
                          timeout=60)
    assert r.ok and r.text == want


# -- the native driver and captured decode steps -----------------------------

@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=str)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_native_driver_equals_python_loop(cases, name, dtype, monkeypatch):
    case = cases(name)
    a, b = tokens_for(case.cfg, 70, 1), tokens_for(case.cfg, 45, 2)
    steps = [[("a", a[:60])], [("a", a[60:61]), ("b", b)], [("a", a[61:])]]
    native = case.engine("cuda:0", dtype)
    assert native.models[case.path].model.use_cpp
    got = feed(native, case.path, steps)
    monkeypatch.setenv("QUORACLE_NO_CPP_FWD", "1")
    loop = case.engine("cuda:0", dtype)
    assert not loop.models[case.path].model.use_cpp
    want = feed(loop, case.path, steps)
    for r in want:
        assert torch.equal(got[r], want[r])


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=str)
def test_captured_decode_equals_eager(cases, dtype):
    """Replays between eager prefills and other work, unread steps included,
    each against the same step run eagerly."""
    case = cases("tiles")
    toks = {r: tokens_for(case.cfg, 80, i) for i, r in enumerate("abc")}
    graph, eager = (case.engine("cuda:0", dtype) for _ in range(2))
    graph.precapture_graphs((1, 2, 4))
    eager.models[case.path].graphs.enabled = False
    at = {r: 0 for r in toks}
    before = 0
    for turn in range(40):
        part = []
        for i, r in enumerate(toks):
            n = 11 if turn in (0, 9 + i, 20) else 1
            if turn % 5 == 4 and r == "b":
                continue
            part.append((r, toks[r][at[r]:at[r] + n]))
            at[r] += n
        part = [(r, t) for r, t in part if t]
        if not part:
            break
        if turn % 3 == 1:                    # nothing wanted, nothing read
            for e in (graph, eager):
                e.step_entries(case.path, [(r, t, ()) for r, t in part],
                               toks)
            continue
        got, want = (e.step_entries(
            case.path, [(r, t, range(len(t))) for r, t in part], toks)
            for e in (graph, eager))
        assert error(got, want) < tolerance(dtype) / 10
        torch.randn(512, 512, device="cuda").sum().item()
        before = graph.stats.get("graph_steps", 0)
    assert before > 20 and "graph_steps" not in eager.stats


# -- the trace runner --------------------------------------------------------

def test_trace_run_protocol(cases, tmp_path):
    """bin/trace_run as a process: the answers, files and line protocol."""
    case = cases("odd")
    toks = tokens_for(case.cfg, 30, 3)
    steps = [
        {"step": 0, "entries": [
            {"id": "a", "tokens": toks[:20], "want": [0, 19]},
            {"id": "b", "tokens": toks[:1], "want": [0]}], "end": ["b"]},
        {"step": 1, "entries": [
            {"id": "a", "tokens": toks[20:29], "want": []}], "end": []},
        {"step": 2, "entries": [
            {"id": "a", "tokens": toks[29:], "want": [0]}], "end": ["a"]}]
    p = subprocess.run(
        [os.path.join(REPO, "bin", "trace_run"), "--model", case.path,
         "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "128",
         "--device", "cpu"],
        input="".join(json.dumps(s) + "\n" for s in steps), text=True,
        capture_output=True, timeout=240)
    assert p.returncode == 0, p.stderr[-2000:]
    done = [x for x in p.stdout.splitlines() if x.startswith("done ")]
    assert done == ["done 0", "done 1", "done 2"]
    assert not (tmp_path / "1.f32").exists()
    want = case.logits(toks)
    for name, places in (("0", [0, 19, 0]), ("2", [29])):
        raw = bytearray((tmp_path / f"{name}.f32").read_bytes())
        got = torch.frombuffer(raw, dtype=torch.float32).view(len(places), -1)
        assert error(got, want[places]) < 2e-5


def test_generate_command(cases):
    case = cases("odd")
    p = subprocess.run(
        [sys.executable, "-m", "quoracle_amd", "generate", "--model",
         case.path, "--prompt", "hi", "--max-tokens", "5", "--dtype",
         "float32", "--device", "cpu", "--kv-gb", "0.01"],
        cwd=REPO, capture_output=True, text=True, timeout=240)
    assert p.returncode == 0, p.stderr[-2000:]
    want = case.engine("cpu", torch.float32).generate_sync(
        request(case, "hi", 5), timeout=60)
    assert p.stdout.rstrip("\n") == want.text.rstrip("\n")
