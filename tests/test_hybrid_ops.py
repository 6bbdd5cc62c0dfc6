"""Each mechanism of the hybrid models alone against its plain equation:
norms, gates, rotation and paged store, chunk-local attention with a sink,
decays, and linear attention in its token-by-token and chunked forms.  On the
CPU these run the plain ops, marked gpu the HIP kernels."""

import math

import pytest
import torch

import koridra_oracle as oracle
from quoracle_amd.models.hybrid_config import RotarySpec
from quoracle_amd.models.llama import ForwardBatch
from quoracle_amd.ops import hybrid as O

F32, BF16 = torch.float32, torch.bfloat16
WHERE = [
    pytest.param(("cpu", F32), id="cpu"),
    pytest.param(("cuda:0", F32), id="gpu-f32", marks=pytest.mark.gpu),
    pytest.param(("cuda:0", BF16), id="gpu-bf16", marks=pytest.mark.gpu),
]


def rand(shape, where, seed=0, gain=1.0):
    """(tensor on the device in its dtype, the same values in float64)."""
    g = torch.Generator().manual_seed(seed)
    t = (torch.randn(*shape, generator=g) * gain).to(where[1])
    return t.to(where[0]), t.double()


def close(got, want, where, tight=2e-5, loose=1e-2):
    got, want = got.detach().cpu().double(), want.double()
    err = float((got - want).norm() / want.norm())
    assert err < (tight if where[1] == F32 else loose), err


def i32(x, dev):
    return torch.tensor(x, dtype=torch.int32, device=dev)


@pytest.mark.parametrize("n", [8, 50, 63, 1032])
@pytest.mark.parametrize("where", WHERE)
def test_embed_and_norms(where, n):
    dev, dt = where
    emb, emb64 = rand((30, n), where, 1)
    pos, pos64 = rand((40, n), where, 2)
    tok, at = i32([3, 29, 0, 3], dev), i32([0, 39, 7, 8], dev)
    x = torch.empty(4, n, device=dev)
    h = torch.empty(4, n, device=dev, dtype=dt)
    O.embed_positions(x, h, emb, pos, tok, at)
    want = emb64[tok.cpu().long()] + pos64[at.cpu().long()]
    close(x, want, (dev, F32))
    close(h, want, where)
    O.embed_positions(x, h, emb, None, tok, at)
    close(x, emb64[tok.cpu().long()], (dev, F32))

    x64 = x.cpu().double()
    a, a64 = rand((4, n), where, 3)
    b, b64 = rand((4, n), where, 4)
    w, w64 = rand((n,), (dev, F32), 5)
    O.post_norm(x, h, a, 0.7, b, -1.2, 1.9, w, 1e-2)
    want = oracle.rms_norm(1.9 * x64 + 0.7 * a64 - 1.2 * b64, w64, 1e-2)
    close(x, want, (dev, F32))
    close(h, want, where)
    x64 = x.cpu().double()
    O.post_norm(x, h, a, 1.0, None, 0.0, 0.3, w, 1e-5)
    close(x, oracle.rms_norm(0.3 * x64 + a64, w64, 1e-5), (dev, F32))

    rows = torch.tensor([2, 0, 2], device=dev)
    out = torch.empty(3, n, device=dev, dtype=dt)
    O.norm_rows(out, x, rows, w, 1e-3)
    close(out, oracle.rms_norm(x.cpu().double()[[2, 0, 2]], w64, 1e-3), where)


@pytest.mark.parametrize("groups,n,off,width", [(1, 96, 8, 200), (5, 11, 3, 61),
                                                (3, 640, 0, 1920)])
@pytest.mark.parametrize("act", [O.ACT_SILU, O.ACT_SIGMOID])
@pytest.mark.parametrize("where", WHERE)
def test_gated_norm(where, act, groups, n, off, width):
    dev, dt = where
    o, o64 = rand((6, groups * n), where, 1)
    proj, p64 = rand((6, width), where, 2)
    w, w64 = rand((n,), (dev, F32), 3)
    out = torch.empty_like(o)
    O.gated_norm(out, o, proj, off, w, groups, act, 1e-3)
    gate = p64[:, off:off + groups * n]
    gate = oracle.silu(gate) if act == O.ACT_SILU else torch.sigmoid(gate)
    y = oracle.rms_norm(o64.view(6, groups, n), w64, 1e-3).reshape(6, -1)
    close(out, y * gate, where)


@pytest.mark.parametrize("n", [64, 37, 2050])
@pytest.mark.parametrize("where", WHERE)
def test_glu(where, n):
    dev, dt = where
    gu, gu64 = rand((5, 2 * n), where, 1, 2.0)
    out = torch.empty(5, n, device=dev, dtype=dt)
    O.glu(out, gu)
    close(out, oracle.silu(gu64[:, :n]) * gu64[:, n:], where)


@pytest.mark.parametrize("rot", [
    {"dims": 8, "base": 100.0},
    {"dims": 2, "base": 10.0,
     "scaling": {"factor": 4.0, "original": 32, "fast": 4.0, "slow": 1.0}},
    {"dims": 64, "base": 10000.0,
     "scaling": {"factor": 16.0, "original": 4096, "fast": 32.0,
                 "slow": 1.0}},
    {"dims": 12, "base": 500.0,        # ramp of no width
     "scaling": {"factor": 2.0, "original": 8, "fast": 1.0, "slow": 1.0}},
], ids=str)
def test_rotary_frequencies(rot):
    sc = rot.get("scaling")
    spec = RotarySpec(rot["dims"], rot["base"], *(
        (sc["factor"], sc["original"], sc["fast"], sc["slow"]) if sc else ()))
    freq, mag = spec.frequencies()
    want, want_mag = oracle.rotary_frequencies(rot)
    assert mag == pytest.approx(want_mag, rel=1e-12)
    assert list(freq) == pytest.approx(want, rel=1e-12)


@pytest.mark.parametrize("H,G,D,dims", [(6, 2, 24, 8), (3, 3, 10, 10),
                                        (2, 1, 7, 4), (4, 2, 64, 0)])
@pytest.mark.parametrize("where", WHERE)
def test_qk_norm_rope_store(where, H, G, D, dims):
    """Norm over the whole projection, rotation of the first dims, rotated
    keys and raw values at their slots, negative slots left alone."""
    dev, dt = where
    T, BS, off = 5, 4, 8
    rot = {"dims": dims, "base": 300.0, "scaling": {
        "factor": 3.0, "original": 64, "fast": 8.0, "slow": 1.0}}
    freq, mag = oracle.rotary_frequencies(rot) if dims else ([], 1.0)
    proj, p64 = rand((T, off + (H + G) * D + 3), where, 1)
    qw, qw64 = rand((H * D,), (dev, F32), 2)
    kw, kw64 = rand((G * D,), (dev, F32), 3)
    positions, slots = [0, 3, 2500, 1, 19], [5, 0, 11, -1, 6]
    q = torch.empty(T, H, D, device=dev, dtype=dt)
    kc = torch.full((3, G, BS, D), 9.0, device=dev, dtype=dt)
    vc = kc.clone()
    O.qk_norm_rope_store(
        q, kc, vc, proj, off, off + H * D, qw, kw, i32(positions, dev),
        i32(slots, dev), torch.tensor(freq, dtype=torch.float64, device=dev),
        mag, 1e-3)
    qn = oracle.rms_norm(p64[:, off:off + H * D], qw64, 1e-3).view(T, H, D)
    raw = p64[:, off + H * D:off + (H + G) * D]
    kn = oracle.rms_norm(raw, kw64, 1e-3).view(T, G, D)

    def turn(x, p):
        return oracle.rotate_interleaved(x, p, rot) if dims else x

    want_k = torch.full((3, G, BS, D), 9.0, dtype=torch.float64)
    want_v = want_k.clone()
    for t, (p, s) in enumerate(zip(positions, slots)):
        close(q[t], torch.stack([turn(qn[t, h], p) for h in range(H)]), where)
        if s >= 0:
            for g in range(G):
                want_k[s // BS, g, s % BS] = turn(kn[t, g], p)
            want_v[s // BS, :, s % BS] = raw.view(T, G, D)[t]
    close(kc, want_k, where)
    assert torch.equal(vc.cpu().double(), want_v)


# -- chunk-local attention ---------------------------------------------------

def paged(k, v, lens, BS, where, seed=0):
    """Scatter sequences' keys/values over shuffled pages."""
    dev, dt = where
    G, D = k[0].shape[1:]
    need = [-(-n // BS) for n in lens]
    order = torch.randperm(sum(need) + 3,
                           generator=torch.Generator().manual_seed(seed))
    kc = torch.full((len(order), G, BS, D), 7.0, dtype=dt)
    vc = torch.full_like(kc, -7.0)
    bt = torch.zeros(len(lens), max(need), dtype=torch.int32)
    at = 0
    for s, n in enumerate(lens):
        bt[s, :need[s]] = order[at:at + need[s]]
        at += need[s]
        for t in range(n):
            kc[bt[s, t // BS], :, t % BS] = k[s][t].to(dt)
            vc[bt[s, t // BS], :, t % BS] = v[s][t].to(dt)
    return kc.to(dev), vc.to(dev), bt.to(dev)


def attention_batch(parts, bt, dev):
    """ForwardBatch of parts [(first position, rows)], single rows first."""
    n_dec = sum(1 for _, n in parts if n == 1)
    tile, row, pos, seq = [[], [], [], []], 0, [], []
    for s, (p, n) in enumerate(parts):
        pos += range(p, p + n)
        seq += [s] * n
        if s >= n_dec:
            for off in range(0, n, O.ATTN_TILE):
                for lst, val in zip(tile, (row + off,
                                           min(O.ATTN_TILE, n - off), s,
                                           p + off)):
                    lst.append(val)
        row += n
    ends = [p + n for p, n in parts]
    return ForwardBatch(
        tokens=i32([0] * row, dev), positions=i32(pos, dev),
        slots=i32([0] * row, dev), block_tables=bt, n_decode=n_dec,
        ctx_lens=i32(ends[:n_dec], dev), max_ctx=max(ends[:n_dec], default=0),
        max_kv=max(ends[n_dec:], default=0), row_seq=i32(seq, dev),
        tile32_q0=i32(tile[0], dev), tile32_qn=i32(tile[1], dev),
        tile32_seq=i32(tile[2], dev), tile32_pos0=i32(tile[3], dev))


def run_attention(where, H, G, D, parts, chunk, sink=True, BS=16, scale=None,
                  shape_inputs=None):
    dev, dt = where
    scale = scale or D ** -0.5
    lens = [p + n for p, n in parts]
    k = [rand((n, G, D), where, 10 + i)[1] for i, n in enumerate(lens)]
    v = [rand((n, G, D), where, 50 + i)[1] for i, n in enumerate(lens)]
    q = rand((sum(n for _, n in parts), H, D), where, 99)[1]
    if shape_inputs:
        shape_inputs(q, k, v)
    q, k = q.to(dt).double(), [x.to(dt).double() for x in k]
    v = [x.to(dt).double() for x in v]
    kc, vc, bt = paged(k, v, lens, BS, where)
    batch = attention_batch(parts, bt, dev)
    out = torch.empty(q.shape, device=dev, dtype=dt)
    O.local_attention(out, q.to(dt).to(dev), kc, vc, batch, scale, chunk,
                      sink)
    want, row = [], 0
    for s, (p, n) in enumerate(parts):
        want.append(oracle.sink_attention(q[row:row + n], k[s], v[s], scale,
                                          chunk, range(p, p + n)))
        row += n
    return out.cpu(), torch.cat(want)


@pytest.mark.parametrize("chunk", [0, 1, 33, 64])
@pytest.mark.parametrize("H,G,D", [(4, 2, 32), (6, 1, 40), (4, 4, 128),
                                   (2, 1, 18), (18, 1, 16), (2, 2, 136)])
@pytest.mark.parametrize("where", WHERE)
def test_local_attention(where, H, G, D, chunk):
    """Decode rows and prefill portions that start and end anywhere, over
    shuffled pages."""
    parts = [(0, 1), (63, 1), (65, 1), (0, 5), (30, 7), (31, 40)]
    got, want = run_attention(where, H, G, D, parts, chunk)
    close(got, want, where)


@pytest.mark.parametrize("where", WHERE)
def test_attention_long_context_splits(where):
    """Contexts long enough that the key walk is split over workgroups."""
    parts = [(1500, 1), (1279, 1), (1290, 20)]
    got, want = run_attention(where, 2, 1, 64, parts, 0)
    close(got, want, where)
    got, want = run_attention(where, 2, 1, 48, parts, 1280)
    close(got, want, where)


@pytest.mark.parametrize("where", WHERE)
def test_sink_only_where_asked(where):
    """Without the sink the weights sum to one; with it they do not."""
    def ones(q, k, v):
        for x in v:
            x.fill_(1.0)
    parts = [(20, 1), (3, 9)]
    plain, _ = run_attention(where, 2, 1, 32, parts, 16, sink=False,
                             shape_inputs=ones)
    close(plain, torch.ones_like(plain).double(), where)
    got, want = run_attention(where, 2, 1, 32, parts, 16, shape_inputs=ones)
    assert float(want.max()) < 0.97
    close(got, want, where)


@pytest.mark.parametrize("key,visible", [
    (96, True), (95, False), (127, True), (112, True), (111, True), (0, False)])
@pytest.mark.parametrize("decoded", [True, False])
@pytest.mark.parametrize("where", WHERE)
def test_one_loud_key(where, decoded, key, visible):
    """One key's score stands far out: it decides the output of a query in
    its chunk (96..127) and is unseen from it when it lies just outside."""
    q_at = 127

    def loud(q, k, v):
        row = q[-1]
        row.zero_()
        row[:, 0] = 8.0
        k[-1][:, :, 0] = 0.0
        k[-1][key, :, 0] = 12.0
        v[-1][key] = 3.0
    parts = [(q_at, 1)] if decoded else [(90, 38)]
    got, want = run_attention(where, 4, 2, 32, parts, 32, shape_inputs=loud)
    assert (abs(float(want[-1].mean()) - 3.0) < 0.05) == visible
    close(got[-1], want[-1], where)


# -- decays ------------------------------------------------------------------

@pytest.mark.parametrize("rank", [1, 16, 21])
@pytest.mark.parametrize("where", WHERE)
def test_log_decay(where, rank):
    """log of sigmoid(.)^(1/tau), also where sigmoid itself underflows; on
    the GPU summed along each chunk where the chunked form reads it."""
    dev, dt = where
    C, T, tau = 48, 9, 3.0
    proj, p64 = rand((T, 40), where, 1, 2.0)
    a2, a64 = rand((C, rank), where, 2, 2.0)
    bias = torch.linspace(-300, 40, C, device=dev)
    out = torch.empty(T, C, device=dev)
    state = torch.empty(2, 2, 8, 24, device=dev)
    batch = ForwardBatch(tokens=i32([0] * T, dev), positions=None, slots=None,
                         block_tables=None, n_decode=2,
                         chunk_row0=i32([2, 6], dev),
                         chunk_len=i32([4, 3], dev))
    O.log_decay(out, proj, 8, a2, bias, tau, batch, state)
    z = p64[:, 8:8 + rank] @ a64.T + bias.cpu().double()
    want = torch.nn.functional.logsigmoid(z) / tau
    if where == ("cuda:0", BF16):
        want[2:6] = want[2:6].cumsum(0)
        want[6:9] = want[6:9].cumsum(0)
    close(out, want, (dev, F32))
    mid = want.abs() < 1
    close(out.cpu()[mid], want[mid], (dev, F32))


# -- linear attention --------------------------------------------------------

def run_linear(where, H, D, V, parts, channel, decay64, act=O.ACT_NONE,
               seed=0):
    """parts [(first position, rows)], single rows first.  The pool starts
    full of noise; a part at position 0 must not see it.  Returns (outputs,
    states) and the oracle's."""
    dev, dt = where
    n_dec = sum(1 for _, n in parts if n == 1)
    T = sum(n for _, n in parts)
    k_off = -(-H * D // 8) * 8
    v_off = 2 * k_off + 8
    proj, p64 = rand((T, -(-(v_off + H * V) // 8) * 8), where, seed, 0.7)
    state, s64 = rand((len(parts) + 2, H, V, D), (dev, F32), seed + 1)
    slots = list(range(len(parts) + 1, 1, -1))
    qscale = D ** -0.5
    seg = {"row0": [], "len": [], "chunk0": [0]}
    chunk = {"row0": [], "len": []}
    row, seq, pos = 0, [], []
    for s, (p, n) in enumerate(parts):
        seq += [s] * n
        pos += range(p, p + n)
        if s >= n_dec:
            seg["row0"].append(row)
            seg["len"].append(n)
            for off in range(0, n, O.LIN_CHUNK):
                chunk["row0"].append(row + off)
                chunk["len"].append(min(O.LIN_CHUNK, n - off))
            seg["chunk0"].append(len(chunk["row0"]))
        row += n
    batch = ForwardBatch(
        tokens=i32([0] * T, dev), positions=i32(pos, dev), slots=None,
        block_tables=None, n_decode=n_dec, row_seq=i32(seq, dev),
        state_slots=i32(slots, dev), seg_row0=i32(seg["row0"], dev),
        seg_len=i32(seg["len"], dev), seg_chunk0=i32(seg["chunk0"], dev),
        chunk_row0=i32(chunk["row0"], dev), chunk_len=i32(chunk["len"], dev))
    powers = None
    if channel:
        ld = decay64.log().reshape(T, H * D)
        if where == ("cuda:0", BF16) and D % 8 == 0 and V % 8 == 0 \
                and D <= 256:
            for r, n in zip(chunk["row0"], chunk["len"]):
                ld[r:r + n] = ld[r:r + n].cumsum(0)
        decay = ld.float().to(dev)
    else:
        d = decay64.view(H)
        decay = d.float().to(dev)
        powers = (d[:, None] ** torch.arange(O.LIN_CHUNK + 1)).float() \
            .contiguous().to(dev)
    o = torch.empty(T, H * V, device=dev, dtype=dt)
    O.linear_attention(o, proj, 0, k_off, v_off, act, qscale, decay, powers,
                       channel, state, batch)

    def part(off, n):
        x = p64[:, off:off + H * n].view(T, H, n)
        return oracle.silu(x) if act == O.ACT_SILU else x
    q, k, v = part(0, D) * qscale, part(k_off, D), part(v_off, V)
    want, want_s, row = [], s64.clone(), 0
    for s, (p, n) in enumerate(parts):
        at = slice(row, row + n)
        d = decay64[at] if channel else decay64.view(1, H, 1)
        start = s64[slots[s]].transpose(1, 2) if p else None
        y, S = oracle.decayed_recurrence(q[at], k[at], v[at], d, start)
        want.append(y.reshape(n, H * V))
        want_s[slots[s]] = S.transpose(1, 2)
        row += n
    return (o.cpu(), state.cpu()), (torch.cat(want), want_s)


PARTS = [(0, 1), (9, 1), (0, 2), (5, 63), (64, 64), (3, 65), (0, 130)]
SIZES = [(2, 16, 24), (3, 64, 32), (1, 72, 136), (2, 128, 64), (3, 10, 13),
         (1, 200, 8), (1, 300, 16)]


@pytest.mark.parametrize("act", [O.ACT_NONE, O.ACT_SILU])
@pytest.mark.parametrize("H,D,V", SIZES)
@pytest.mark.parametrize("where", WHERE)
def test_linear_attention_head_decay(where, H, D, V, act):
    decay = torch.tensor([1.0, 0.93, 0.2][:H], dtype=torch.float64)
    got, want = run_linear(where, H, D, V, PARTS, False, decay, act)
    close(got[0], want[0], where)
    # the state is float32 in both modes: what differs is the rounding of
    # activated inputs
    close(got[1], want[1], where, loose=4e-3)


@pytest.mark.parametrize("strong", [False, True])
@pytest.mark.parametrize("H,D,V", SIZES)
@pytest.mark.parametrize("where", WHERE)
def test_linear_attention_channel_decay(where, H, D, V, strong):
    """Decays near one, and decays that wipe a channel within a step or two
    beside channels that keep everything."""
    T = sum(n for _, n in PARTS)
    g = torch.Generator().manual_seed(5)
    z = torch.rand(T, H, D, generator=g, dtype=torch.float64)
    decay = 0.9 + 0.1 * z
    if strong:
        decay = torch.where(z < 0.3, 1e-30, torch.where(z < 0.6, 1.0, decay))
    got, want = run_linear(where, H, D, V, PARTS, True, decay)
    close(got[0], want[0], where, loose=6e-3)
    # strong: log decays of -69 a step sum to over a thousand in a chunk, and
    # a float32 of that size resolves 1e-4 of a logarithm
    close(got[1], want[1], where, loose=2e-4 if strong else 2e-5)


@pytest.mark.parametrize("channel", [False, True])
@pytest.mark.parametrize("where", WHERE)
def test_a_far_key_through_the_state(where, channel):
    """One loud early key, no decay: a query 300 tokens later, all others
    silent, reads its value back through five chunks of state."""
    dev, dt = where
    H, D, V, T = 1, 32, 16, 300
    proj = torch.zeros(T, 2 * D + V, dtype=dt)
    proj[7, D + 3] = 4.0
    proj[7, 2 * D:] = torch.arange(V).to(dt)
    proj[T - 1, 3] = 2.0
    starts = list(range(0, T, O.LIN_CHUNK))
    batch = ForwardBatch(
        tokens=i32([0] * T, dev), positions=i32(range(T), dev), slots=None,
        block_tables=None, n_decode=0, row_seq=i32([0] * T, dev),
        state_slots=i32([1], dev), seg_row0=i32([0], dev),
        seg_len=i32([T], dev), seg_chunk0=i32([0, len(starts)], dev),
        chunk_row0=i32(starts, dev),
        chunk_len=i32([min(O.LIN_CHUNK, T - s) for s in starts], dev))
    state = torch.full((2, H, V, D), 5.0, device=dev)
    decay = torch.zeros(T, D, device=dev) if channel \
        else torch.ones(H, device=dev)
    powers = torch.ones(H, O.LIN_CHUNK + 1, device=dev)
    o = torch.empty(T, V, device=dev, dtype=dt)
    O.linear_attention(o, proj.to(dev), 0, D, 2 * D, O.ACT_NONE, 1.0, decay,
                       powers, channel, state, batch)
    o = o.cpu().double()
    assert torch.equal(o[:T - 1], torch.zeros(T - 1, V).double())
    assert torch.equal(o[T - 1], 8.0 * torch.arange(V).double())
    assert math.isclose(float(state[1].sum()),
                        4.0 * sum(range(V)), rel_tol=1e-6)
    assert float(state[0].min()) == 5.0          # another slot is untouched
