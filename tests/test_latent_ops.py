"""Each mechanism of latent attention, mixtures of experts and the norms around
a sublayer alone against its plain equation.  On the CPU these run the plain
ops, marked gpu the HIP kernels."""

import pytest
import torch

import kotutar_oracle as oracle
from quoracle_amd.models.hybrid_config import LatentAttentionSpec, RotarySpec
from quoracle_amd.models.llama import ForwardBatch
from quoracle_amd.ops import latent as L

F32, BF16, F64 = torch.float32, torch.bfloat16, torch.float64
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


def frequencies(dims, base, dev):
    return torch.tensor(RotarySpec(dims, base).frequencies()[0],
                        dtype=F64, device=dev)


# -- norms -------------------------------------------------------------------

# more values than a workgroup holds in registers, and sizes no vector takes
@pytest.mark.parametrize("n", [8, 50, 63, 1032, 5000, 9000, 1025])
@pytest.mark.parametrize("where", WHERE)
def test_pre_norm(where, n):
    dev, dt = where
    x, x64 = rand((4, n), (dev, F32), 1)
    y, y64 = rand((4, n), (dev, F32), 2)
    w, w64 = rand((n,), (dev, F32), 3)
    h = torch.empty(4, n, device=dev, dtype=dt)
    L.pre_norm(x, h, None, w, 1e-2)
    close(h, oracle.rms_norm(x64, w64, 1e-2), where)
    close(x, x64, (dev, F32), 1e-12)
    L.pre_norm(x, h, y, w, 1e-2)
    close(h, oracle.rms_norm(y64, w64, 1e-2), where)
    close(x, y64, (dev, F32), 1e-12)


@pytest.mark.parametrize("n", [8, 50, 63, 1032, 5000, 9000, 1025])
@pytest.mark.parametrize("terms,bias,second", [(1, True, False),
                                               (1, False, False),
                                               (3, False, True)])
@pytest.mark.parametrize("where", WHERE)
def test_sandwich_norm(where, n, terms, bias, second):
    dev, dt = where
    T = 5
    x, x64 = rand((T, n), (dev, F32), 1)
    y, y64 = rand((T, terms, n) if terms > 1 else (T, n), where, 2)
    w, w64 = rand((n,), (dev, F32), 3)
    nxt, n64 = rand((n,), (dev, F32), 4)
    b, b64 = rand((n,), (dev, F32), 5)
    y2, y264 = rand((T, n), where, 6)
    gate, g64 = rand((T,), (dev, F32), 7)
    s = y64.sum(1) if terms > 1 else y64
    if bias:
        s = s + b64
    if second:
        s = s + g64[:, None] * y264
    want = x64 + oracle.rms_norm(s, w64, 1e-2)
    h = torch.empty(T, n, device=dev, dtype=dt)
    joined = torch.full((T, 2 * n), 3.0, device=dev, dtype=dt)
    start = x.clone()
    args = (y, b if bias else None, y2 if second else None,
            gate if second else None, w, 1e-2)
    L.sandwich_norm(x, h, None, nxt, *args)
    close(x, want, (dev, F32))
    close(h, oracle.rms_norm(want, n64, 1e-2), where)
    # in front of a pass: the stream goes to the first half of `joined`
    h.fill_(9.0)
    L.sandwich_norm(start, h, joined, None, *args)
    close(start, want, (dev, F32))
    close(joined[:, :n], want, where)
    assert bool((joined[:, n:] == 3).all()) and bool((h == 9).all())


# -- latents into the cache --------------------------------------------------

@pytest.mark.parametrize("q_rank,rank,rot", [(48, 72, 16), (9, 5, 2),
                                             (21, 19, 6), (640, 512, 64),
                                             (1536, 24, 8)])
@pytest.mark.parametrize("where", WHERE)
def test_latent_store(where, q_rank, rank, rot):
    """Both norms, the rotated part unnormed, everything at its slot; the
    padding of the pool's rows stays zero, negative slots are left alone."""
    dev, dt = where
    T, BS = 5, 4
    pad = [n + -n % 8 for n in (q_rank, rank, rot)]
    width = pad[1] + pad[2]
    proj, p64 = rand((T, pad[0] + rank + rot + -(rank + rot) % 8), where, 1)
    wq, wq64 = rand((q_rank,), (dev, F32), 2)
    wkv, wkv64 = rand((rank,), (dev, F32), 3)
    positions, slots = [0, 3, 70000, 1, 19], [5, 0, 11, -1, 6]
    if dev == "cpu":
        slots[3] = 9
    cq = torch.empty(T, q_rank, device=dev, dtype=dt)
    pool = torch.zeros(3, BS, width, device=dev, dtype=dt)
    L.latent_store(cq, pool, proj, pad[0], pad[1], wq, wkv,
                   i32(positions, dev), i32(slots, dev),
                   frequencies(rot, 300.0, dev), 1e-2)
    close(cq, oracle.rms_norm(p64[:, :q_rank], wq64, 1e-2), where)
    want = torch.zeros(3 * BS, width, dtype=F64)
    c = oracle.rms_norm(p64[:, pad[0]:pad[0] + rank], wkv64, 1e-2)
    for t, (p, s) in enumerate(zip(positions, slots)):
        if s >= 0:
            want[s, :rank] = c[t]
            want[s, pad[1]:pad[1] + rot] = oracle.rotate(
                p64[t, pad[0] + rank:pad[0] + rank + rot], p, rot, 300.0)
    close(pool.view(-1, width), want, where)
    assert bool((pool.view(-1, width).cpu()[want == 0] == 0).all())


@pytest.mark.parametrize("H,off,rot,D", [(3, 24, 16, 40), (5, 10, 6, 18),
                                         (2, 8, 2, 16), (1, 0, 64, 64)])
@pytest.mark.parametrize("where", WHERE)
def test_rotate_heads(where, H, off, rot, D):
    dev, dt = where
    positions = [0, 1, 5, 999, 100000]
    q, q64 = rand((5, H, D), where, 1)
    L.rotate_heads(q, off, i32(positions, dev), frequencies(rot, 1e4, dev))
    want = q64.clone()
    for t, p in enumerate(positions):
        want[t, :, off:off + rot] = oracle.rotate(
            q64[t, :, off:off + rot], p, rot, 1e4)
    close(q, want, where)
    outside = [d for d in range(D) if not off <= d < off + rot]
    assert torch.equal(q.cpu().double()[:, :, outside],
                       q64[:, :, outside])


# -- attention ---------------------------------------------------------------

QT, BIG = 16, 128


def spec(H, D, R, V, rank):
    return LatentAttentionSpec(H, D, R, V, 8, rank, 1.0, RotarySpec(R, 1e4))


def make_batch(parts, bt, BS, dev, split):
    """ForwardBatch of parts [(first position, rows)]: single rows first,
    then portions shorter than `split` (None: no difference), then others."""
    n_dec = sum(1 for _, n in parts if n == 1)
    short, big = [[], [], [], []], [[], [], [], []]
    row, pos, seq, slots, ctx0 = 0, [], [], [], []
    n_latent = n_dec
    for s, (p, n) in enumerate(parts):
        pos += range(p, p + n)
        seq += [s] * n
        if s >= n_dec:
            is_short = split is not None and n < split
            lists, step = (short, QT) if is_short else (big, BIG)
            for off in range(0, n, step):
                for lst, val in zip(lists, (row + off, min(step, n - off), s,
                                            p + off)):
                    lst.append(val)
                if not is_short and split is not None:
                    ctx0.append(len(slots))
            if is_short:
                n_latent = row + n
            elif split is not None:
                slots += [int(bt[s, t // BS]) * BS + t % BS
                          for t in range(p + n)]
        row += n
    ends = [p + n for p, n in parts]
    tiles = {}
    for name, lists in (("tile", short), ("tile32", big)):
        for k, lst in zip(("q0", "qn", "seq", "pos0"), lists):
            tiles[f"{name}_{k}"] = i32(lst, dev) if lst else None
    return ForwardBatch(
        tokens=i32([0] * row, dev), positions=i32(pos, dev),
        slots=i32([0] * row, dev), block_tables=bt.to(dev), n_decode=n_dec,
        ctx_lens=i32(ends[:n_dec], dev), max_ctx=max(ends[:n_dec], default=0),
        max_kv=max(ends[n_dec:], default=0), row_seq=i32(seq, dev),
        n_latent=n_latent, ctx_slots=i32(slots, dev) if slots else None,
        tile32_ctx0=i32(ctx0, dev) if ctx0 else None, **tiles)


def attend(where, H, D, R, V, rank, parts, split=24, sink=True, BS=16,
           scale=None, shape=None):
    """(framework's output, oracle's) over shuffled pages; `shape` may change
    the inputs: shape(q, c, k_rot, sink)."""
    dev, dt = where
    sp = spec(H, D, R, V, rank)
    scale = scale or 1.5 * (D + R) ** -0.5
    q = rand((sum(n for _, n in parts), H, D + R), where, 1)[1]
    lens = [p + n for p, n in parts]
    c = [rand((n, rank), where, 10 + i)[1] for i, n in enumerate(lens)]
    kr = [rand((n, R), where, 60 + i)[1] for i, n in enumerate(lens)]
    uk = rand((H, D, rank), where, 2, rank ** -0.5)[1]
    uv = rand((H, V, rank), where, 3, rank ** -0.5)[1]
    sk = rand((H,), (dev, F32), 4)[1] + 1.0
    if shape:
        shape(q, c, kr, sk)
    q = q.to(dt)
    need = [-(-n // BS) for n in lens]
    order = torch.randperm(sum(need) + 3,
                           generator=torch.Generator().manual_seed(5))
    pool = torch.full((len(order), BS, sp.cache_width), 7.0, dtype=dt)
    bt = torch.zeros(len(lens), max(need), dtype=torch.int32)
    at = 0
    for s, n in enumerate(lens):
        bt[s, :need[s]] = order[at:at + need[s]]
        at += need[s]
        for t in range(n):
            line = pool[bt[s, t // BS], t % BS]
            line.zero_()
            line[:rank] = c[s][t].to(dt)
            line[sp.rank_p:sp.rank_p + R] = kr[s][t].to(dt)
    # what the kernels read: parts padded with zeros
    def pad(x, *sizes):
        out = torch.zeros(*x.shape[:-len(sizes)], *sizes, dtype=x.dtype)
        out[tuple(slice(0, n) for n in x.shape)] = x
        return out
    qp = torch.cat([pad(q[..., :D], sp.dim_p), pad(q[..., D:], sp.rot_p)], -1)
    uk_p = pad(uk.to(dt), sp.dim_p, sp.rank_p)
    uv_p = pad(uv.to(dt), sp.vdim_p, sp.rank_p)
    w_kv = torch.cat([uk_p.flatten(0, 1), uv_p.flatten(0, 1)])
    if not L.tiles_ok(sp, dt):
        split = None
    elif not L.expandable(sp):
        split = 1 << 30
    batch = make_batch(parts, bt, BS, dev, split)
    out = torch.empty(q.shape[0], H, sp.vdim_p, device=dev, dtype=dt)
    L.latent_attention(
        out, qp.contiguous().to(dev), pool.to(dev), w_kv.to(dev),
        uk_p.transpose(1, 2).contiguous().to(dev),
        sk.float().to(dev) if sink else None, scale, batch)
    want, row = [], 0
    sk = sk if sink else torch.full_like(sk, -1e9)
    for s, (p, n) in enumerate(parts):
        k = torch.cat([torch.einsum("tr,hdr->thd", c[s], uk),
                       kr[s][:, None].expand(-1, H, -1)], -1)
        v = torch.einsum("tr,hvr->thv", c[s], uv)
        want.append(oracle.attend(q[row:row + n].double(), k, v, scale, sk,
                                  range(p, p + n)))
        row += n
    assert not out[..., V:].any()
    return out[..., :V].cpu(), torch.cat(want)


PARTS = [(0, 1), (63, 1), (65, 1), (0, 5), (30, 7), (47, 20), (31, 40),
         (0, 24), (100, 150)]
SIZES = [(5, 24, 16, 40, 72), (1, 16, 8, 16, 64), (18, 64, 64, 128, 136),
         (3, 40, 40, 64, 256), (2, 192, 64, 248, 264), (33, 32, 8, 32, 512),
         (4, 128, 64, 128, 512), (3, 10, 6, 13, 19), (2, 200, 64, 264, 72),
         (2, 16, 72, 24, 520), (7, 8, 2, 8, 8)]


@pytest.mark.parametrize("H,D,R,V,rank", SIZES)
@pytest.mark.parametrize("where", WHERE)
def test_latent_attention(where, H, D, R, V, rank):
    """Decode rows, short portions and long ones that start and end anywhere,
    over shuffled pages."""
    got, want = attend(where, H, D, R, V, rank, PARTS)
    close(got, want, where)


@pytest.mark.parametrize("parts", [[(9, 1)], [(9, 1), (70, 1)], [(0, 2)],
                                   [(0, 60)], [(7, 1), (0, 60)],
                                   [(7, 1), (0, 2)], [(0, 2), (0, 60)]],
                         ids=str)
@pytest.mark.parametrize("where", WHERE)
def test_batches_of_every_kind(where, parts):
    got, want = attend(where, 5, 24, 16, 40, 72, parts)
    close(got, want, where)


@pytest.mark.parametrize("H", [2, 6, 40])
@pytest.mark.parametrize("where", WHERE)
def test_long_context_splits(where, H):
    """Contexts long enough that the key walk is split over workgroups."""
    parts = [(1500, 1), (1279, 1), (1290, 9), (1100, 40), (2, 2), (3, 50)]
    got, want = attend(where, H, 16, 8, 24, 40, parts)
    close(got, want, where)


@pytest.mark.parametrize("parts", [[(20, 1)], [(3, 9)], [(3, 40)]], ids=str)
@pytest.mark.parametrize("where", WHERE)
def test_sink(where, parts):
    """A large sink takes most of the weight, once; without it the weights
    sum to one."""
    def level(q, c, kr, sk):
        q.zero_()                            # all scores 0
        sk.copy_(torch.tensor([3.0, -2.0]))
        for x in c:
            x[:] = x[0]                      # all values alike
    got, want = attend(where, 2, 16, 8, 24, 40, parts, shape=level)
    close(got, want, where)
    plain, free = attend(where, 2, 16, 8, 24, 40, parts, sink=False,
                         shape=level)
    close(plain, free, where)
    keys = parts[0][0] + 1
    for h, s in enumerate((3.0, -2.0)):
        share = keys / (keys + torch.tensor(s).exp())
        close(got[0, h], free[0, h] * share, where)


@pytest.mark.parametrize("at,seen", [(0, True), (15, True), (16, True),
                                     (63, True), (64, True), (127, True),
                                     (128, False)])
@pytest.mark.parametrize("part", [(127, 1), (120, 9), (90, 60), (0, 150)],
                         ids=str)
@pytest.mark.parametrize("loud", ["latent", "rotated"])
@pytest.mark.parametrize("where", WHERE)
def test_one_loud_key(where, loud, part, at, seen):
    """One key's score stands far out, by its latent or by its rotated part:
    it decides the output of the query at 127, and is unseen from there when
    it comes later."""
    if at >= sum(part):
        pytest.skip("past the end")
    D, R, rank = 16, 8, 40
    row = 127 - part[0]

    def shape(q, c, kr, sk):
        q[row] = 0.0
        for x in kr:
            x[:, 0] = 0.0
        if loud == "rotated":
            q[row, :, D] = 10.0
            kr[0][at, 0] = 12.0
        else:
            # a query that picks out the direction of one latent
            q[row, :, :D] = 6.0 * torch.einsum(
                "hdr,r->hd", rand((2, D, rank), where, 2, rank ** -0.5)[1],
                c[0][at]).sign()
    got, want = attend(where, 2, D, R, 24, rank, [part], shape=shape)
    # scores this large carry the rounding of the query further
    close(got[row], want[row], where, loose=2e-2)
    close(got, want, where, loose=2e-2)
    uv = rand((2, 24, rank), where, 3, rank ** -0.5)[1]
    alone = torch.einsum("hvr,r->hv", uv, rand(
        (sum(part), rank), where, 10)[1][at])
    if loud == "rotated":
        near = float((want[row] - alone).norm() / alone.norm()) < 0.05
        assert near == seen


# -- feed-forwards -----------------------------------------------------------

@pytest.mark.parametrize("n", [64, 37, 2050, 2056])
@pytest.mark.parametrize("bias", [True, False])
@pytest.mark.parametrize("where", WHERE)
def test_bias_gelu(where, n, bias):
    dev, dt = where
    z, z64 = rand((5, n), where, 1, 2.0)
    b, b64 = rand((n,), (dev, F32), 2)
    L.bias_gelu(z, b if bias else None)
    close(z, oracle.gelu(z64 + b64 if bias else z64), where)


def test_gelu_is_the_exact_form():
    """Far from the tanh form: by nearly 1e-4 around 2, not by rounding."""
    z = torch.tensor([[2.0, -2.0, 0.5, -4.0]])
    tanh = torch.nn.functional.gelu(z.double(), approximate="tanh")
    want = oracle.gelu(z.double())
    L.bias_gelu(z, None)
    assert float((z - want).abs().max()) < 1e-6
    assert float((tanh - want).abs().max()) > 5e-5


@pytest.mark.parametrize("n,E,top", [(80, 7, 2), (54, 3, 3), (40, 1, 1),
                                     (136, 70, 8), (1024, 130, 1),
                                     (64, 400, 5), (50, 65, 6)])
@pytest.mark.parametrize("T", [1, 16, 37])
@pytest.mark.parametrize("gated", [True, False])
@pytest.mark.parametrize("where", WHERE)
def test_moe_route(where, n, E, top, T, gated):
    dev, _ = where
    h, h64 = rand((T, n), where, 1)
    r, r64 = rand((E + gated, n), where, 2, n ** -0.5)
    ids = torch.full((T, top), -1, dtype=torch.int32, device=dev)
    w = torch.empty(T, top, device=dev)
    gate = torch.empty(T, device=dev) if gated else None
    L.moe_route(ids, w, gate, h, r, E)
    s = torch.sigmoid(h64 @ r64.T)
    picks = s[:, :E].gather(1, ids.cpu().long())
    close(w, picks, (dev, F32))
    # the largest, each once (equal up to a float32 rounding)
    best = s[:, :E].topk(top).values
    assert float((picks - best).abs().max()) < 1e-6
    assert all(len(set(row)) == top for row in ids.tolist())
    if gated:
        close(gate, s[:, E], (dev, F32))


@pytest.mark.parametrize("n,ff,E,top", [(80, 56, 7, 2), (54, 33, 3, 3),
                                        (40, 24, 1, 1), (136, 48, 70, 3),
                                        (264, 200, 4, 1), (64, 520, 5, 4)])
@pytest.mark.parametrize("T", [1, 5, 70, 300])
@pytest.mark.parametrize("uneven", [False, True])
@pytest.mark.parametrize("where", WHERE)
def test_moe_experts(where, n, ff, E, top, T, uneven):
    """The weight on the input; experts with many rows, one and none."""
    dev, dt = where
    h, h64 = rand((T, n), where, 1)
    up, up64 = rand((E, ff, n), where, 2, n ** -0.5)
    down, down64 = rand((E, n, ff), where, 3, ff ** -0.5)
    g = torch.Generator().manual_seed(4)
    first = torch.zeros(T, dtype=torch.long) if uneven else \
        torch.randint(0, E, (T,), generator=g)
    ids = (first[:, None] + torch.arange(top)) % E
    w = torch.rand(T, top, generator=g) + 0.2
    y = torch.empty(T, top, n, device=dev, dtype=dt)
    L.moe_experts(y, h, ids.int().to(dev), w.to(dev), up, down)
    want = torch.empty(T, top, n, dtype=F64)
    W = {f"{e}.{k}": m[e] for e in range(E)
         for k, m in (("up", up64), ("down", down64))}
    for t in range(T):
        for k in range(top):
            want[t, k] = oracle.expert(w[t, k].double() * h64[t], W,
                                       f"{int(ids[t, k])}.")
    close(y, want, where)


@pytest.mark.gpu
@pytest.mark.parametrize("n", [16, 50, 1024])
@pytest.mark.parametrize("dtype", [F32, BF16], ids=str)
def test_linear_f32(n, dtype):
    """A product with a float32 result keeps what bf16 would round off."""
    a, a64 = rand((7, n), ("cuda:0", dtype), 1)
    w, w64 = rand((24, n), ("cuda:0", dtype), 2)
    got = L.linear_f32(a, w)
    assert got.dtype == F32
    close(got, a64 @ w64.T, ("cuda:0", F32))


def test_expansion_threshold():
    """Between 16 and 256; higher where making keys and values costs more
    than it saves."""
    big = spec(32, 128, 64, 128, 512)
    assert 16 <= big.expand_from < 256
    assert spec(2, 64, 8, 64, 64).expand_from == 256
    assert spec(2, 8, 8, 8, 512).expand_from == 16
