"""The kernels that Pokepel added to the serving library, each against the
plain implementation: retention on rotated keys, latent attention with a sink
and neighbouring pairs, gated branches of the residual, polynomial
activations, softmax routing over the best groups."""

import math

import pytest
import torch

import pokepel_oracle as po
from neuronx_distributed_amd.ops import serving as sv

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [F32, BF16]
TOL = {F32: 1e-5, BF16: 8e-3}


@pytest.fixture(scope="module", autouse=True)
def _built():
    sv.ensure_built()


def _rand(*shape, seed=0, dtype=F32, scale=1.0):
    g = torch.Generator().manual_seed(seed + sum(shape))
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device="cuda")


def _near(got, want, dtype, what="", tol=None):
    """Largest error, row by row, over the largest value of the row."""
    got, want = got.double().cpu(), want.double()
    assert got.shape == want.shape and torch.isfinite(got).all(), what
    top = want.abs().amax(dim=-1, keepdim=True)
    err = (got - want).abs() / top.clamp(min=1e-3 * want.abs().max().item())
    assert err.max() < (tol or TOL[dtype]), (what, err.max().item())


# ---------------------------------------------------------------------------
# retention
# ---------------------------------------------------------------------------

# H, D, E, elements that turn
RETENTION = [
    (3, 40, 24, 32), (2, 64, 128, 64), (4, 72, 48, 72), (2, 24, 136, 8),
    (2, 128, 128, 48), (1, 136, 160, 128), (2, 200, 64, 24), (2, 256, 96, 256),
    (3, 13, 7, 6), (1, 6, 33, 6), (2, 16, 8, 0), (1, 320, 40, 320),
]
DECAYS = [0.9995, 0.9, 1.0, 0.99]


def _turn_gate(H, D, rot):
    d = sv.decay_gate(DECAYS[:H], "cuda")
    return sv.TurnGate(d.decay, d.log2_decay, D ** -0.5,
                       sv.rotary_frequencies(rot["base"], rot["dims"],
                                             "cuda"))


def _prepared(q, k, H, D, rot):
    T = q.shape[0]
    turned = [po.rotate_halves(x.double().view(T, H, D), range(T), rot)
              for x in (q, k)]
    return turned[0], turned[1] * D ** -0.5


class Requests:
    """Two requests of T tokens, fed side by side in portions."""

    def __init__(self, H, D, E, dims, T, dtype):
        self.H, self.D, self.E, self.T = H, D, E, T
        self.rot = {"base": 500.0, "dims": dims}
        self.x = [[_rand(T, H * n, seed=10 * i + j, dtype=dtype)
                   for j, n in enumerate((D, D, E, E))] for i in range(2)]
        self.want, self.state = [], []
        for q, k, v, _ in self.x:
            o, S = po.retention(*_prepared(q, k, H, D, self.rot),
                                v.double().view(T, H, E), DECAYS[:H])
            self.want.append(o.reshape(T, H * E))
            self.state.append(S)
        self.gate = _turn_gate(H, D, self.rot)

    def feed(self, cuts, chunked, gated=False, eps=1e-2):
        S = torch.full((5, self.H, self.D, self.E), 1e4, device="cuda")
        at, got = 0, []
        for n in cuts:
            seg = [(3, 0, n, at), (1, n, n, at)]
            chunks, first = sv.chunk_table(seg)
            # strided, as slices of one product
            rows = torch.cat([torch.cat([t[at:at + n] for t in x], 1)
                              for x in self.x]).cuda()
            q, k, v, g = rows.split([t.shape[1] for t in self.x[0]], 1)
            kw = dict(chunks=_i32(chunks), chunk_first=_i32(first)) \
                if chunked else {}
            if gated:
                kw.update(silu_gate=g, eps=eps)
            o = sv.memory_mix(q, k, v, self.gate, S, None, None, _i32(seg),
                              self.H, **kw)
            got.append(o.view(2, n, -1))
            at += n
        return torch.cat(got, 1), S


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", RETENTION)
def test_retention_in_portions(case, dtype):
    """Every cut gives the whole sequence's output and state, from slots that
    held something else."""
    T = 330
    r = Requests(*case, T, dtype)
    for cuts in ([T], [2] * 15 + [300], [256, 74], [64, 1, 63, 129, 73],
                 [255, 2, 73]):
        for chunked in (False, True):
            got, S = r.feed(cuts, chunked)
            for i, slot in enumerate((3, 1)):
                what = (case, cuts[:3], chunked, i)
                _near(got[i], r.want[i], dtype, what, 3 * TOL[dtype])
                _near(S[slot].flatten(0, 1), r.state[i].flatten(0, 1), F32,
                      what, 2e-5 if dtype == F32 or not chunked else 1e-4)
            assert (S[[0, 2, 4]] == 1e4).all()


@pytest.mark.parametrize("case", RETENTION[:8])
def test_retention_keeps_rotated_keys_beyond_bf16(case):
    """The chunk kernels' state is that of the unrounded rotated keys; one
    rounding to bf16 would show a hundredfold."""
    H, D, E, dims = case
    r = Requests(*case, 200, BF16)
    _, S = r.feed([200], True)
    q, k = _prepared(r.x[0][0], r.x[0][1], H, D, r.rot)
    _, rounded = po.retention(q, k.bfloat16().double(),
                              r.x[0][2].double().view(200, H, E), DECAYS[:H])
    off = (rounded - r.state[0]).pow(2).mean().sqrt()
    err = (S[3].double().cpu() - r.state[0]).pow(2).mean().sqrt()
    assert err < off / 50, (err.item(), off.item())


@pytest.mark.parametrize("case", [c for c in RETENTION if c[1] % 8 == 0])
def test_retention_norms_and_gates_its_heads(case):
    H, D, E, dims = case
    T, eps = 300, 1e-2
    r = Requests(*case, T, BF16)
    probe = r.x[0][0].cuda()
    fits = r.gate.norm_fits(BF16, D, E, probe)
    assert fits == (D <= 128 and E <= 128 or D <= 256 and E <= 64)
    if not fits:
        return
    for cuts in ([T], [40, 2, 258]):
        got, _ = r.feed(cuts, True, True, eps)
        for i in range(2):
            want = po.rms(r.want[i].view(T, H, E), eps).reshape(T, -1) * \
                po.silu(r.x[i][3].double())
            _near(got[i].view(T * H, E), want.view(T * H, E), BF16,
                  (case, cuts, i), 3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_retention_far_key_and_chunk_borders(dtype):
    """A head that forgets nothing: one large key stands out for all later
    tokens, in prompts and decoding, wherever chunks end."""
    H, D, E, T = 2, 32, 16, 700
    rot = {"base": 1e6, "dims": 32}
    gate = sv.TurnGate(*(lambda d: (d.decay, d.log2_decay))(
        sv.decay_gate([1.0, 0.9999], "cuda")), D ** -0.5,
        sv.rotary_frequencies(rot["base"], rot["dims"], "cuda"))
    for spot in (0, 1, 63, 64, 255, 256, 511, 512, 600):
        q, k, v = (_rand(T, H * n, seed=i, dtype=dtype, scale=0.05)
                   for i, n in enumerate((D, D, E)))
        k[spot] = _rand(H * D, seed=9, dtype=dtype) * 8
        v[spot] = _rand(H * E, seed=8, dtype=dtype) * 8
        qr, kr = _prepared(q, k, H, D, rot)
        want, _ = po.retention(qr, kr, v.double().view(T, H, E),
                               [1.0, 0.9999])
        want = want.reshape(T, -1)
        cuda = [t.cuda() for t in (q, k, v)]
        for cuts in ([T], [256, 444], [690] + [1] * 10, [spot + 1, T - spot - 1]):
            S = torch.full((2, H, D, E), -77.0, device="cuda")
            at = 0
            for n in cuts:
                seg = [(1, 0, n, at)]
                chunks, first = sv.chunk_table(seg)
                kw = dict(chunks=_i32(chunks), chunk_first=_i32(first)) \
                    if n > 1 else {}
                o = sv.memory_mix(*(t[at:at + n] for t in cuda), gate, S,
                                  None, None, _i32(seg), H, **kw)
                # later tokens see it, earlier ones do not
                sel = slice(max(at, spot), at + n)
                if sel.start < sel.stop:
                    # 700 products of a rounded decay, and sums that cancel
                    _near(o[sel.start - at:], want[sel], dtype,
                          (spot, cuts[:2], at),
                          2e-4 if dtype == F32 else 3e-2)
                if at < spot:
                    early = min(n, spot - at)
                    w = want[at:at + early]
                    err = (o[:early].double().cpu() - w).abs().max()
                    assert err < 1e-2 * want[spot:].abs().max()
                at += n


def test_retention_far_positions_turn_exactly():
    """Single tokens at large positions: a state of one known key."""
    H, D, E = 1, 16, 8
    rot = {"base": 100.0, "dims": 12}
    gate = _turn_gate(H, D, rot)
    for p in (1, 4097, 131071, 1000003):
        q, k, v = (_rand(1, n, seed=i, dtype=F32) for i, n in
                   enumerate((D, D, E)))
        S = torch.zeros(1, H, D, E, device="cuda")
        o = sv.memory_mix(q.cuda(), k.cuda(), v.cuda(), gate, S, None, None,
                          _i32([(0, 0, 1, p)]), H)
        kr = po.rotate_halves(k.double().view(1, 1, D), [p], rot)[0, 0]
        want = kr[:, None] * D ** -0.5 * v.double()
        _near(S[0, 0], want, F32, p)
        qr = po.rotate_halves(q.double().view(1, 1, D), [p], rot)[0, 0]
        _near(o, (qr @ want)[None], F32, p)


def test_retention_refuses_what_does_not_fit():
    H, D, E = 2, 16, 8
    q, v = torch.zeros(2, H * D).cuda(), torch.zeros(2, H * E).cuda()
    S = torch.zeros(1, H, D, E).cuda()
    seg = _i32([(0, 0, 2, 0)])
    wide = _turn_gate(H, D, {"base": 9.0, "dims": 18})
    with pytest.raises(ValueError):
        sv.memory_mix(q, q, v, wide, S, None, None, seg, H)
    with pytest.raises(AssertionError):       # gates belong to the chunks
        sv.memory_mix(q, q, v, _turn_gate(H, D, {"base": 9.0, "dims": 16}),
                      S, None, None, seg, H, silu_gate=v)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,group", [(3, 24), (1, 33), (4, 128),
                                         (2, 2048)])
def test_silu_gated_norm_without_weight(heads, group, dtype):
    T, N, eps = 5, heads * group, 1e-3
    o, z = _rand(T, N, dtype=dtype), _rand(T, N + 8, seed=1, dtype=dtype)
    want = po.rms(o.double().view(T, heads, group), eps).reshape(T, N) * \
        po.silu(z[:, :N].double())
    x = o.cuda()
    _near(sv.gated_norm(x, None, z.cuda()[:, :N], group, eps, True), want,
          dtype)
    y = x.clone()
    sv.gated_norm(y[2:], None, z.cuda()[2:, :N], group, eps, True, out=y[2:])
    _near(y[2:], want[2:], dtype)
    assert torch.equal(y[:2], x[:2])


# ---------------------------------------------------------------------------
# latent attention
# ---------------------------------------------------------------------------

class Step:
    """The fields of a step of one request that latent attention reads."""

    def __init__(self, ctx, n, bt, expand):
        self.pos, self.seq = _i32(list(range(ctx, ctx + n))), _i32([0] * n)
        self.block_table, self.max_keys = bt, ctx + n
        self.portion_tokens = n if n > 1 else 0
        self.tiles = _i32([(0, s, min(128, n - s), ctx + s)
                           for s in range(0, n, 128)])
        self.spans = {}
        if n > 1 and expand:
            pages, table = sv.key_spans([(0, 0, n, ctx)], bt.tolist(), 0)
            self.spans = {0: sv.KeySpans(_i32(pages), _i32(table))}


# H, dim, rot, vdim, rank
LATENT = [
    (4, 32, 16, 24, 48), (36, 16, 16, 16, 136), (2, 128, 64, 128, 512),
    (3, 10, 6, 7, 21), (2, 40, 80, 200, 600), (2, 112, 48, 96, 64),
    (5, 24, 8, 80, 256), (1, 8, 64, 8, 960),
]


def _latent_case(H, D, P, E, R, T, dtype, spot=None):
    """Queries, rows, gates, weights and the answer; ``spot``: the latent of
    that token stands out for every query."""
    rot = {"base": 300.0, "dims": P, "scaling": {
        "factor": 4.0, "original": 60, "fast": 4.0, "slow": 0.5}}
    q = _rand(T, H * (D + P), dtype=dtype)
    kv = _rand(T, R + P, dtype=dtype, seed=1)
    gate = _rand(T, H * E, dtype=dtype, seed=2)
    sink = _rand(H, dtype=dtype, seed=3, scale=2.0)
    norm = (1 + _rand(R, seed=5, scale=0.2)).to(dtype)
    uk = _rand(H * D, R, dtype=dtype, seed=6, scale=R ** -0.5)
    uv = _rand(H * E, R, dtype=dtype, seed=7, scale=R ** -0.5)
    if spot is not None:
        uk[::D, :] = 0.0
        uk[::D, 0] = 1.0
        kv[:, 0] = 0.0
        kv[spot, 0] = 3.0 * R ** 0.5
        q.view(T, H, D + P)[..., 0] = 5.0 * R ** 0.25
    freq, amp = sv.yarn_frequencies(300.0, P, "cuda", rot["scaling"])
    w = sv.LatentWeights(
        norm.cuda(), uk.view(H, D, R).transpose(1, 2).contiguous().cuda(),
        torch.cat([uk, uv]).cuda(), freq, amp, True, sink.cuda())
    cfg = {"heads": H, "dim": D, "rot_dim": P, "vdim": E, "kv_rank": R,
           "scale": 1.3 * (D + P) ** -0.5, "rot": rot}
    d = torch.float64
    c, kr = po.latents(kv.to(d), norm.to(d), R, rot, range(T), 1e-5)
    want = po.latent_attention(q.to(d), c, kr, uk.to(d), uv.to(d), sink.to(d),
                               cfg, range(T)) * po.sigmoid(gate.to(d))
    return q, kv, gate, w, cfg, want


def _cache(T, width, dtype, seed=0):
    """Scattered pages full of large stale values, and their table."""
    n = -(-T // 64)
    perm = torch.randperm(n + 1, generator=torch.Generator().manual_seed(seed))
    return torch.full((n + 1, 64, width), 77.0, dtype=dtype).cuda(), \
        perm.int().view(1, -1).cuda()


def _attend(q, kv, gate, w, cfg, cuts, expand, dtype, seed=0):
    cache, bt = _cache(q.shape[0], kv.shape[1], dtype, seed)
    out, at = [], 0
    for n in cuts:
        s = slice(at, at + n)
        out.append(sv.latent_attention(
            q[s].cuda(), kv[s].cuda(), gate[s].cuda(),
            Step(at, n, bt, expand), cache, w, cfg["heads"], cfg["dim"],
            cfg["vdim"], cfg["scale"], 1e-5))
        at += n
    return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", LATENT)
def test_latent_attention_with_sinks_and_pairs(case, dtype):
    T = 210
    q, kv, gate, w, cfg, want = _latent_case(*case, T, dtype)
    for expand in (True, False):
        for cuts in ([T], [2, 62, 64, 3, 50, 29], [130] + [1] * 80,
                     [1, 1, 2, 1, 63, 2, 140]):
            got = _attend(q, kv, gate, w, cfg, cuts, expand, dtype, len(cuts))
            _near(got, want, dtype, (case, expand, cuts[:4]),
                  2e-5 if dtype == F32 else 2.5e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_one_split_counts_the_sink(dtype):
    """A long context shared by many workgroups, sinks that take nearly
    everything and nearly nothing; and the first token."""
    H, D, P, E, R, T = 4, 16, 8, 16, 32, 1500
    q, kv, gate, w, cfg, _ = _latent_case(H, D, P, E, R, T, dtype)
    w.sink = torch.tensor([9.0, -50.0, 0.0, 7.5], dtype=dtype).cuda()
    d = torch.float64
    c, kr = po.latents(kv.to(d), w.norm.cpu().to(d), R, cfg["rot"], range(T),
                       1e-5)
    full = w.expand.cpu().to(d)
    want = po.latent_attention(q.to(d), c, kr, full[:H * D], full[H * D:],
                               w.sink.cpu().to(d), cfg, range(T)) * \
        po.sigmoid(gate.to(d))
    got = _attend(q, kv, gate, w, cfg, [T - 5] + [1] * 5, True, dtype)
    got, want = (x.view(T * H, E) for x in (got, want))   # head by head
    _near(got, want, dtype, tol=2e-5 if dtype == F32 else 3e-2)
    share = want[-4:].abs().mean(1)
    assert share[0] < share[1] / 3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("spot", [0, 1, 63, 64, 127, 128, 300])
def test_far_latents_show(spot, dtype):
    """One latent stands out for every later query, across pages."""
    T = 400
    q, kv, gate, w, cfg, want = _latent_case(3, 16, 8, 24, 40, T, dtype, spot)
    other = _latent_case(3, 16, 8, 24, 40, T, dtype, spot + 2)[5]
    assert (want - other)[spot + 2:].abs().max() > 0.3
    for cuts in ([T], [spot + 2, T - spot - 2], [390] + [1] * 10):
        for expand in (True, False):
            got = _attend(q, kv, gate, w, cfg, cuts, expand, dtype)
            _near(got, want, dtype, (spot, cuts[:2], expand),
                  3e-5 if dtype == F32 else 3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_pairs_turn_exactly_far_out(dtype):
    H, D, P, R = 2, 6, 12, 20
    rot = {"base": 10000.0, "dims": 8, "scaling": {
        "factor": 6.0, "original": 1000, "fast": 8.0, "slow": 1.0}}
    where = [0, 1, 63, 64, 5000, 131071]
    T = len(where)
    q = _rand(T, H * (D + P), dtype=dtype)
    kv = _rand(T, R + P, dtype=dtype, seed=3)
    cache = torch.zeros(T, 64, R + P, dtype=dtype).cuda()
    bt = torch.zeros(T, 131072 // 64, dtype=torch.int32)
    for t, p in enumerate(where):
        bt[t, p // 64] = t
    w = sv.LatentWeights(torch.ones(R, dtype=dtype).cuda(), None, None,
                         *sv.yarn_frequencies(1e4, 8, "cuda", rot["scaling"]),
                         True)
    qc = q.cuda()
    sv.latent_append(qc, D, D + P, qc, D, D + P, kv.cuda(), w, cache,
                     _i32(where), _i32(list(range(T))), bt.cuda(), H, 1e-3)

    want = po.rotate_pairs(q.double().view(T, H, D + P)[..., D:], where, rot)
    got = qc.view(T, H, D + P)
    _near(got[..., D:], want, dtype)
    assert torch.equal(got[..., :D].cpu(), q.view(T, H, D + P)[..., :D])
    rows = torch.stack([cache[t, p % 64] for t, p in enumerate(where)])
    _near(rows[:, R:], po.rotate_pairs(kv[:, R:].double(), where, rot), dtype)


# ---------------------------------------------------------------------------
# gated branches of the residual
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,W,parts", [(3, 50, 2), (5, 128, 1),
                                          (70, 264, 3), (2, 4096, 6),
                                          (600, 2048, 5)])
def test_gated_branches(rows, W, parts, dtype):
    """One or two branches, with each of their pieces and without it."""
    d = torch.float64
    x = _rand(rows, W)
    y1 = _rand(rows, W, seed=1, dtype=dtype)
    y2 = _rand(rows * parts, W, seed=2, dtype=dtype)
    coef = torch.rand(rows, parts)
    plus = _rand(rows, W, seed=3, dtype=dtype)
    gates = _rand(rows, 2 * W + 8, seed=4, dtype=dtype)
    b1, b2 = (_rand(W, seed=s, dtype=dtype) for s in (5, 6))
    w = _rand(W, seed=7, dtype=dtype)
    g1, g2 = gates[:, :W], gates[:, W + 8:]
    gc = gates.cuda()
    sig = lambda g, b: po.sigmoid(g.to(d) + b.to(d))
    first = y1.to(d) * sig(g1, b1)
    mixed = (y2.to(d).view(rows, parts, W) * coef.to(d)[..., None]).sum(1)
    A = sv.Branch(y1.cuda(), gate=gc[:, :W], bias=b1.cuda())
    c = dict(coef=coef.cuda())
    cases = [
        ([A], first),
        ([A, sv.Branch(y2.cuda(), **c, plus=plus.cuda(), gate=gc[:, W + 8:],
                       bias=b2.cuda())],
         first + (mixed + plus.to(d)) * sig(g2, b2)),
        ([A, sv.Branch(y2.cuda(), **c, gate=gc[:, W + 8:])],
         first + mixed * po.sigmoid(g2.to(d))),
        ([sv.Branch(y2.cuda(), **c), sv.Branch(plus.cuda())],
         mixed + plus.to(d)),
    ]
    pick = torch.tensor([rows - 1, 0, rows - 1])
    for branches, add in cases:
        for base in (x, None):
            new = add + (0 if base is None else x.to(d))
            b = None if base is None else x.cuda()
            got, h, _ = sv.residual_norm(b, sv.Pending(branches=branches),
                                         1e-3, w.cuda())
            _near(got, new, F32)
            _near(h, po.norm(new, w.to(d), 1e-3), dtype)
            _, h, _ = sv.residual_norm(b, sv.Pending(branches=branches), 1e-3,
                                       w.cuda(), keep_x=False,
                                       index=pick.int().cuda())
            _near(h, po.norm(new, w.to(d), 1e-3)[pick], dtype)
    vec = _rand(W, seed=8, dtype=dtype)
    got, _, _ = sv.residual_norm(x.cuda(), sv.Pending(
        branches=[A], vec=vec.cuda()), 1e-3, w.cuda())
    _near(got, x.to(d) + first + vec.to(d), F32)


# ---------------------------------------------------------------------------
# feed-forwards
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,n", [(1, 1), (3, 77), (9, 4096), (2, 16384),
                                 (2, 20000), (1, 16385), (300, 96)])
def test_poly_norm(T, n, dtype):
    x = _rand(T, n + 8, dtype=dtype) * torch.linspace(0.1, 2, n + 8)
    x = x.to(dtype)
    x[0, 0] = 9.0
    act = torch.tensor([0.7, -0.4, 0.9, 0.25]).to(dtype)
    want = po.poly_norm(x[:, :n].double(), act.double(), 1e-2)
    got = sv.poly_norm(x.cuda()[:, :n], act.cuda(), 1e-2)
    _near(got, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,n", [(1, 1), (7, 77), (70000, 4), (5, 4096)])
def test_silu_mul(T, n, dtype):
    x = _rand(T, 2 * n + 4, dtype=dtype)
    got = sv.silu_mul(x.cuda()[:, :2 * n])
    _near(got, po.silu(x[:, :n].double()) * x[:, n:2 * n].double(), dtype)


@pytest.mark.parametrize("T,E,count,keep,top", [
    (1, 8, 2, 1, 2), (5, 6, 3, 2, 4), (64, 64, 8, 3, 6), (65, 130, 10, 2, 20),
    (300, 512, 64, 5, 7), (33, 7, 7, 3, 1), (9, 5, 1, 1, 5),
    (40, 12, 4, 4, 3)])
def test_softmax_routing_over_best_groups(T, E, count, keep, top):
    z = _rand(T, E, scale=2.0)
    r = sv.Routing(top, groups=count, keep=keep, softmax=True, best=1)
    p = sv.moe_plan(z.cuda(), None, r, 0)
    idx, w = po.route(z.double(), count, keep, top)
    assert torch.equal(p.idx.cpu().long(), idx)
    _near(p.coef, w, F32)
    assert E == top or (p.coef.sum(1) < 1 - 1e-6).any()
    assert sorted(p.order.tolist()) == list(range(T * top))


def test_routing_takes_large_logits():
    z = torch.tensor([[300.0, 299.0, -300.0, 0.0]])
    p = sv.moe_plan(z.cuda(), None, sv.Routing(3, softmax=True), 0)
    assert p.idx.tolist() == [[0, 1, 3]]
    _near(p.coef, torch.softmax(z.double(), 1)[:, [0, 1, 3]], F32)
    with pytest.raises(ValueError):
        sv.moe_plan(z.cuda(), None, sv.Routing(2, groups=2, best=3), 0)
    with pytest.raises(ValueError):
        sv.moe_plan(z.cuda(), None, sv.Routing(2, True, softmax=True), 0)
