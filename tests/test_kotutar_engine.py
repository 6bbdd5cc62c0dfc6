"""Kotutar through the engine against the plain oracle: whole prompts,
token-by-token decoding, portions, mixed batches, reused pages, loud far keys,
and generation by the scheduler.  The same tests run on the CPU (plain ops)
and, marked gpu, on the HIP kernels in float32 and bf16."""

import json
import os
import subprocess
import sys

import pytest
import torch

import kotutar_oracle as oracle
from hybrid_cases import (cut, error, feed, greedy, paced, request, tokens_for,
                          tolerance, write_checkpoint)
from kotutar_cases import CONFIGS, Case, random_weights

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
def test_routers_make_no_close_call(cases, name):
    """What the bf16 comparisons rest on."""
    case, margins = cases(name), []
    route = oracle.route

    def spy(h, W, p, router):
        z = (h @ W[p + "router"].T).sort(-1, descending=True).values
        if router["top"] < router["experts"]:
            margins.append((z[:, router["top"] - 1]
                            - z[:, router["top"]]).min())
        return route(h, W, p, router)
    oracle.route = spy
    try:
        oracle.forward(case.cfg, case.weights, tokens_for(case.cfg, 150, 150))
    finally:
        oracle.route = route
    assert all(m > 0.1 for m in margins), margins


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
def test_stream_after_every_run(cases, name, where):
    """The residual stream behind each layer run, looped layers included."""
    case = cases(name)
    toks = tokens_for(case.cfg, 37, 3)
    eng = case.engine(*where)
    model, got = eng.models[case.path].model, []
    good = model.forward
    model.forward = lambda batch, kv: good(batch, kv, stream=got)
    feed(eng, case.path, [[("a", toks)]])
    want = oracle.forward(case.cfg, case.weights, toks)[1]
    assert len(got) == len(want)
    for x, y in zip(got, want):
        assert error(x.cpu(), y) < tolerance(where[1])


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


@pytest.mark.parametrize("sizes", [[2], [3, 2, 17], [64, 1, 63], [37, 36, 1],
                                   [19, 20, 21, 16, 15]], ids=str)
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
    """Unequal requests side by side, some decoding, some in short and some
    in long portions, one paused; then new ones in the pages that were given
    back, with a pool that does not hold all of them at once."""
    case = cases(name)
    lens = {"a": 90, "b": 33, "c": 5, "d": 110, "e": 64, "f": 90}
    reqs = {r: tokens_for(case.cfg, n, 7 * n + i)
            for i, (r, n) in enumerate(lens.items())}
    sizes = {"a": [20, 1, 1, 9], "b": [2, 1], "c": [1], "d": [50, 3, 1],
             "e": [16], "f": [1, 31]}
    parts = {r: cut(reqs[r], sizes[r]) for r in reqs}
    eng = case.engine(*where, blocks=20, slots=3)
    eng.precapture_graphs((1, 2, 4))
    got = feed(eng, case.path, paced(parts, 3))
    check(case, got, reqs, where[1])
    assert eng.models[case.path].mgr.free_blocks == 19


@pytest.mark.parametrize("where", WHERE)
def test_short_and_long_portions_in_one_batch(cases, where):
    """Portions just below and just above the length from which keys and
    values are made from the whole context, beside single tokens."""
    case = cases("tiles")
    eng = case.engine(*where)
    split = eng.models[case.path].model.expand_from or 20
    assert 2 < split < 100
    lens = {"a": split, "b": 1, "c": split - 1, "d": 2 * split, "e": 2}
    reqs = {r: tokens_for(case.cfg, n + split + 9, n)
            for r, n in lens.items()}
    got = feed(eng, case.path, [
        [(r, reqs[r][:n]) for r, n in lens.items()],
        [(r, reqs[r][n:n + k]) for (r, n), k
         in zip(lens.items(), (1, split - 1, split, 2, 39))],
        [(r, reqs[r][n + k:]) for (r, n), k
         in zip(lens.items(), (1, split - 1, split, 2, 39))]])
    check(case, got, reqs, where[1])


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

def _without(name, cfg, weights):
    cfg, weights = json.loads(json.dumps(cfg)), dict(weights)
    if name == "sink":
        for k in weights:
            if k.endswith(".sink"):
                weights[k] = torch.full_like(weights[k], -1e4)
    elif name == "a pass":
        cfg["loop"]["times"] -= 1
    elif name == "shared expert":
        for x in cfg["layers"]:
            if x["mlp"]:
                x["mlp"].pop("shared", None)
    elif name == "rotation":
        for x in cfg["layers"]:
            x["mixer"]["rot"]["base"] *= 1.1
    elif name == "biases":
        for k in weights:
            if k.endswith(".b"):
                weights[k] = torch.zeros_like(weights[k])
    return cfg, weights


@pytest.mark.parametrize("what", ["sink", "a pass", "shared expert",
                                  "rotation", "biases", "the last key",
                                  "the first key", "input weights"])
def test_oracle_shows_a_wrong_mechanism(cases, what, monkeypatch):
    """A small mistake moves the logits by far more than the tolerance, so
    the comparisons above would show it."""
    case = cases("tiles")
    toks = tokens_for(case.cfg, 60, 9)
    right = case.logits(toks)
    if what == "the last key":
        monkeypatch.setattr(oracle, "sees", lambda i, j: j < max(i, 1))
    elif what == "the first key":
        monkeypatch.setattr(oracle, "sees", lambda i, j: min(i, 1) <= j <= i)
    elif what == "input weights":
        def late(h, W, p, m):
            """The weight on the output instead."""
            out = torch.zeros_like(h)
            for t, picks in enumerate(oracle.route(h, W, p, m["router"])):
                for e, w in picks:
                    out[t] += w * oracle.expert(h[t], W, f"{p}e{e}.")
            return out + oracle.moe_ff(h, W, p, dict(m, router={
                **m["router"], "top": 0}))
        monkeypatch.setitem(oracle.FEED_FORWARD, "moe", late)
    wrong = oracle.forward(*_without(what, case.cfg, case.weights), toks)[0]
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
        [{"role": "user", "content": "a portion's border lies in this"}])
    want = greedy(case, prompt, 12)
    r = eng.generate_sync(
        request(case, "a portion's border lies in this", 12), timeout=120)
    assert r.ok, r.error
    assert r.output_tokens == len(want)
    assert r.text == eng.tokenizer.decode([t for t in want if t != 257])


@pytest.mark.parametrize("where", WHERE[:2])
def test_requests_together_as_alone(cases, where):
    """Five requests in a pool that cannot hold them all at once come out as
    they do alone, and everything is given back."""
    case = cases("odd")
    texts = ["one", "number two", "3", "the fourth request", "v"]
    alone = {t: case.engine(*where).generate_sync(
        request(case, t, 9), timeout=120).text for t in texts}
    eng = case.engine(*where, blocks=14)
    done = {}
    for t in texts:
        eng._submit(request(case, t, 9),
                    ("cb", lambda r, t=t: done.__setitem__(t, r)))
    for _ in range(400):
        if len(done) == len(texts):
            break
        eng.step()
    assert {t: r.text for t, r in done.items()} == alone
    assert not eng.models[case.path].active


@pytest.mark.parametrize("where", WHERE[:2])
def test_session_reuses_its_prefix(cases, where):
    """Latents of a shared prefix stay; a diverging tail is cut off.  The text
    is the same as in a fresh engine."""
    case = cases("tiles")
    eng = case.engine(*where)
    for i, text in enumerate(("hello there", "hello there", "hello you")):
        got = eng.generate_sync(request(case, text, 6, session_id="s"),
                                timeout=120)
        fresh = case.engine(*where).generate_sync(request(case, text, 6),
                                                  timeout=120)
        assert got.text == fresh.text
        assert (eng.stats["prefix_hit_tokens"] > 0) == (i > 0)


def test_bad_input_is_refused(cases):
    case = cases("odd")
    eng = case.engine("cpu", torch.float32, blocks=10)
    with pytest.raises(ValueError):
        eng.step_entries(case.path, [("a", [case.cfg["vocab"]], [])])
    with pytest.raises(ValueError):
        eng.step_entries(case.path, [("a", [-1], [])])
    with pytest.raises(ValueError):
        eng.step_entries(case.path, [("a", [1], [1])])


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
@pytest.mark.parametrize("name", ["tiles", "wide"])
def test_captured_decode_equals_eager(cases, name, dtype):
    """Replays between eager prefills and other work, unread steps included,
    each against the same step run eagerly."""
    case = cases(name)
    toks = {r: tokens_for(case.cfg, 80, i) for i, r in enumerate("abc")}
    graph, eager = (case.engine("cuda:0", dtype) for _ in range(2))
    graph.precapture_graphs((1, 2, 4))
    eager.models[case.path].graphs.enabled = False
    at = {r: 0 for r in toks}
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
        assert error(got, want) < tolerance(dtype) / 3
        torch.randn(512, 512, device="cuda").sum().item()
    assert graph.stats.get("graph_steps", 0) > 20
    assert "graph_steps" not in eager.stats


# -- commands ----------------------------------------------------------------

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


def test_preset_by_name():
    """Random weights of a preset, hosted by its name."""
    from quoracle_amd.engine.engine import LocalEngine
    eng = LocalEngine(["kotutar-tiny"], device=torch.device("cpu"),
                      embed_model_key=None, kv_blocks_override=40,
                      dtype=torch.float32)
    hm = eng.models["kotutar-tiny"]
    assert len(hm.model.runs) == 6 and len(hm.kv.latent) == 6
    lg = eng.step_entries("kotutar-tiny", [("a", [5, 6, 7], [0, 2])])
    assert lg.shape == (2, 512) and bool(torch.isfinite(lg).all())


# -- configuration -----------------------------------------------------------

def test_config_counts(cases):
    from quoracle_amd.models import get_config
    case = cases("tiles")
    cfg = get_config(case.path)
    shapes = cfg.tensor_shapes()
    assert {k: tuple(w.shape) for k, w in case.weights.items()} == shapes
    assert [r.layer for r in cfg.runs()] == [0, 1, 2, 1, 2, 1, 2, 3]
    assert [r.latent for r in cfg.runs()] == list(range(8))
    assert [r.enter for r in cfg.runs()] == [False, True, False, True, False,
                                             True, False, False]
    hm = case.engine("cpu", torch.float32).models[case.path]
    per_token = cfg.kv_bytes_per_token(4)
    assert hm.kv.bytes() == 96 * 16 * per_token
    assert not cfg.needs_state


@pytest.mark.parametrize("change", [
    lambda c: c["layers"][0].update(type="other"),
    lambda c: c["layers"][0]["mlp"].update(kind="other"),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=8),
    lambda c: c["layers"][1]["mlp"]["router"].update(top=8),
    lambda c: c["loop"].update(stop=5)])
def test_bad_configurations_are_refused(change):
    from quoracle_amd.models.hybrid_config import KotutarConfig
    cfg = json.loads(json.dumps(CONFIGS["tiles"]))
    KotutarConfig.from_dict(cfg)
    change(cfg)
    with pytest.raises(ValueError):
        KotutarConfig.from_dict(cfg)


def test_wrong_shapes_are_refused(tmp_path):
    cfg = json.loads(json.dumps(CONFIGS["odd"]))
    weights = random_weights(cfg)
    weights["l0.mix.uk"] = weights["l0.mix.uk"][:-1]
    from quoracle_amd.models import build_model
    path = write_checkpoint(str(tmp_path), cfg, weights)
    with pytest.raises(ValueError, match="l0.mix.uk"):
        build_model(path, torch.device("cpu"), torch.float32)
