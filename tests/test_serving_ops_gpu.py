"""Serving kernels on the GPU, each against the plain implementation in
``voletar_oracle`` (float64), one mechanism at a time."""

import math

import pytest
import torch

import voletar_oracle as vo

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module", autouse=True)
def sv():
    from neuronx_distributed_amd.ops import serving

    serving.ensure_built()
    return serving


def _close(got, want, dtype, scale=1.0, what=""):
    got, want = got.detach().double().cpu(), want.double()
    assert torch.isfinite(got).all(), what
    tol = (3e-6 if dtype == torch.float32 else 6e-3) * scale
    err = (got - want).abs() / want.abs().amax(dim=-1, keepdim=True).clamp(
        min=1e-3)
    assert err.max().item() < tol, (what, err.max().item(), tol)


def _rand(*shape, dtype, scale=1.0, seed=0):
    g = torch.Generator().manual_seed(seed + sum(shape))
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


# ---------------------------------------------------------------------------
# attention
# ---------------------------------------------------------------------------

class Paged:
    """Requests of given lengths over scattered pages of a cache that is
    full of large stale values."""

    def __init__(self, lengths, G, D, E, dtype, seed=0):
        gen = torch.Generator().manual_seed(seed)
        per = [-(-n // 64) for n in lengths]
        pages = sum(per) + 2
        perm = torch.randperm(pages, generator=gen).int()
        self.bt = torch.full((len(lengths), max(per) + 1), int(perm[-1]),
                             dtype=torch.int32)
        at = 0
        for r, n in enumerate(per):
            self.bt[r, :n] = perm[at:at + n]
            at += n
        self.bt = self.bt.cuda()
        self.kc = torch.full((pages, G, 64, D), 77.0, dtype=dtype).cuda()
        self.vc = torch.full((pages, G, 64, E), -55.0, dtype=dtype).cuda()


ATTN = [
    # H, G, D, E, window, keep
    (4, 2, 56, 64, 90, 21),
    (6, 2, 40, 24, 70, 5),
    (3, 1, 20, 12, 33, 0),        # sizes that are no multiple of 8
    (8, 8, 128, 96, 130, 130),
    (16, 2, 96, 128, 64, 64),
    (2, 2, 200, 256, 65, 1),
    (4, 4, 32, 48, 0, 0),         # plain causal
    (10, 2, 16, 16, 1, 3),
]


def _attn_case(H, G, D, E, window, keep, T, dtype, seed=1):
    q = _rand(T, H * D, dtype=dtype, seed=seed)
    k = _rand(T, G * D, dtype=dtype, seed=seed + 1)
    v = _rand(T, G * E, dtype=dtype, seed=seed + 2)
    mask = {"size": window, "keep_first": keep} if window else None
    want = vo.windowed_attention(
        q.double().view(T, H, D), k.double().view(T, G, D),
        v.double().view(T, G, E), 0.11, mask).reshape(T, H * E)
    return q, k, v, want


def _portions(sv, c, q, k, v, cuts, H, window, keep, req=0):
    """Feed one request in portions; a portion of one token decodes."""
    outs, at = [], 0
    for n in cuts:
        qs, ks, vs = (t[at:at + n].cuda() for t in (q, k, v))
        pos = torch.arange(at, at + n, dtype=torch.int32).cuda()
        seq = torch.full((n,), req, dtype=torch.int32).cuda()
        kw = dict(heads=H, scale=0.11, window=window, keep=keep,
                  max_keys=at + n)
        if n == 1:
            o = sv.attn_rows(qs, ks, vs, c.kc, c.vc, pos, seq, c.bt, **kw)
        else:
            tiles = torch.tensor(
                [(req, s, min(128, n - s), at + s) for s in range(0, n, 128)],
                dtype=torch.int32).cuda()
            o = sv.attn_portions(qs, ks, vs, c.kc, c.vc, pos, seq, c.bt,
                                 tiles, **kw)
        outs.append(o)
        at += n
    assert at == q.shape[0]
    return torch.cat(outs)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", ATTN)
def test_attention_prompt_portions_and_decoding(sv, case, dtype):
    H, G, D, E, window, keep = case
    T = 290
    q, k, v, want = _attn_case(*case, T, dtype)
    for cuts in ([T], [2, 62, 64, 3, 129, 30], [130] + [1] * 160,
                 [1, 1, 2, 1, 63, 2, 200, 20]):
        c = Paged([T], G, D, E, dtype, seed=len(cuts))
        got = _portions(sv, c, q, k, v, cuts, H, window, keep)
        _close(got, want, dtype, what=(case, cuts[:4]))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep", [(92, 22), (64, 64), (70, 3),
                                         (33, 0), (128, 65)])
def test_attention_edges_show(sv, window, keep, dtype):
    """One key stands out; queries just inside see it, just outside do not.
    The planted places: the last kept token, the first that is not kept,
    page borders, and the window's edge of several queries."""
    H, G, D, E, T = 4, 2, 64, 32, 330
    spots = sorted({0, max(keep - 1, 0), keep, keep + 1, 63, 64, 65, 127,
                    128, 200})
    mask = {"size": window, "keep_first": keep}
    for s in spots:
        q = _rand(T, H * D, dtype=dtype, seed=3)
        k = _rand(T, G * D, dtype=dtype, seed=4, scale=0.3)
        v = _rand(T, G * E, dtype=dtype, seed=5)
        q[:, 0::D] = 8.0                       # first dim of every head
        k[:, 0::D] = 0.0
        k[s, 0::D] = 14.0                      # score + 12 at this key
        v[s] = 6.0
        want = vo.windowed_attention(
            q.double().view(T, H, D), k.double().view(T, G, D),
            v.double().view(T, G, E), 0.11, mask)
        seen = torch.tensor([vo.visible(i, s, mask) for i in range(T)])
        assert (want.mean((1, 2))[seen] > 5).all()       # it shows
        if (~seen).any():
            assert (want.mean((1, 2))[~seen] < 2).all()
        for cuts in ([T], [keep + 2] + [1] * (T - keep - 2)):
            c = Paged([T], G, D, E, dtype, seed=s)
            got = _portions(sv, c, q, k, v, cuts, H, window, keep)
            _close(got, want.reshape(T, H * E), dtype,
                   what=(window, keep, s, cuts[0]))


@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_batch_of_unequal_requests(sv, dtype):
    H, G, D, E, window, keep = 6, 3, 48, 32, 50, 7
    lens = [3, 140, 64, 257]
    c = Paged(lens, G, D, E, dtype)
    data = [_attn_case(H, G, D, E, window, keep, n, dtype, seed=20 + n)
            for n in lens]
    kw = dict(heads=H, scale=0.11, window=window, keep=keep, max_keys=257)
    # all but the last token of every request in one call, then one each
    q, k, v = (torch.cat([d[i][:-1] for d in data]).cuda() for i in range(3))
    pos, seq, tiles, at = [], [], [], 0
    for r, n in enumerate(lens):
        for s in range(0, n - 1, 128):
            tiles.append((r, at + s, min(128, n - 1 - s), s))
        pos += range(n - 1)
        seq += [r] * (n - 1)
        at += n - 1
    i32 = lambda x: torch.tensor(x, dtype=torch.int32).cuda()
    got = sv.attn_portions(q, k, v, c.kc, c.vc, i32(pos), i32(seq), c.bt,
                           i32(tiles), **kw)
    _close(got, torch.cat([d[3][:-1] for d in data]), dtype)
    q, k, v = (torch.cat([d[i][-1:] for d in data]).cuda() for i in range(3))
    got = sv.attn_rows(q, k, v, c.kc, c.vc, i32([n - 1 for n in lens]),
                       i32(range(4)), c.bt, **kw)
    _close(got, torch.cat([d[3][-1:] for d in data]), dtype)


def test_attention_weights_keep_32_bits(sv):
    """Two far apart values under nearly equal weights: bf16 weights would
    lose the small one's contribution to the sum of many."""
    H, G, D, E, T = 1, 1, 32, 32, 128
    q = torch.zeros(T, D, dtype=torch.bfloat16)
    q[:, 0] = 1
    k = torch.zeros(T, D, dtype=torch.bfloat16)
    k[:, 0] = (torch.arange(T) % 7).to(torch.bfloat16) * 0.37
    v = torch.full((T, E), 1.0, dtype=torch.bfloat16)
    v[1::2] = -1.0
    want = vo.windowed_attention(q.double()[:, None], k.double()[:, None],
                                 v.double()[:, None], 0.11, None)[:, 0]
    c = Paged([T], G, D, E, torch.bfloat16)
    got = _portions(sv, c, q, k, v, [T], 1, 0, 0).double().cpu()
    # rows where the signs nearly cancel: the error of the weights decides
    small = want[:, 0].abs() < 0.02
    assert small.sum() > 20
    assert ((got - want).abs()[small] <
            2e-5 + 4e-3 * want.abs()[small]).all()


# ---------------------------------------------------------------------------
# matrix memories
# ---------------------------------------------------------------------------

MEM = [(4, 56, 40), (3, 48, 72), (2, 20, 12), (2, 128, 96), (1, 256, 40),
       (5, 8, 8), (1, 300, 34)]


def _mem_inputs(H, D, E, T, dtype, seed=0):
    # one fused projection, read as strided slices
    pad = 8 - (2 * H * D + H * E) % 8
    p = _rand(T, 2 * H * D + H * E + pad, dtype=dtype, seed=seed)
    return p[:, :H * D], p[:, H * D:2 * H * D], p[:, 2 * H * D:][:, :H * E], p


def _tables(sv, seg, chunked):
    i32 = lambda x: torch.tensor(x, dtype=torch.int32).cuda()
    return (i32(seg), *map(i32, sv.chunk_table(seg))) if chunked \
        else (i32(seg),)


def _run_memory(sv, proj, sizes, cuts, H, gate_of, S, n, m, slot):
    outs, at = [], 0
    for c in cuts:
        part = proj[at:at + c].cuda()
        a, b, w = sizes
        q, k, v = part[:, :a], part[:, a:a + b], part[:, a + b:a + b + w]
        seg = [(slot, 0, c, at)]
        outs.append(sv.memory_mix(q, k, v, gate_of(at, c), S, n, m,
                                  *_tables(sv, seg, c > 1)[:1], H,
                                  *_tables(sv, seg, c > 1)[1:]))
        at += c
    return torch.cat(outs)


T_MEM = 600
CUTS = ([T_MEM], [64, 2, 190, 3, 257, 84], [500] + [1] * 100,
        [1, 1, 2, 256, 128, 212], [255, 256, 89])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,E", MEM)
def test_decayed_memory(sv, H, D, E, dtype):
    T = T_MEM
    decay = [0.0, 1.0, 0.97, 0.6, 0.999][:H] if H > 2 else [0.998, 0.5][:H]
    q, k, v, p = _mem_inputs(H, D, E, T, dtype, seed=7)
    d = lambda t, s: vo.silu(t.double()).view(T, H, s)
    if dtype == torch.bfloat16:   # activations may round to bf16
        d = lambda t, s: vo.silu(t.double()).to(dtype).double().view(T, H, s)
    want, S_want = vo.decayed_memory(d(q, D), d(k, D), d(v, E),
                                     torch.tensor(decay).double())
    gate = sv.decay_gate(decay, "cuda")
    for cuts in CUTS:
        S = torch.full((3, H, D, E), 1e4).cuda()   # a slot used before
        got = _run_memory(sv, p, (H * D, H * D, H * E), cuts, H,
                          lambda at, c: gate, S, None, None, slot=2)
        _close(got, want.reshape(T, H * E), dtype, 2.0, (H, D, E, cuts[:4]))
        err = (S[2].double().cpu() - S_want).abs().max() / S_want.abs().max()
        assert err < (2e-5 if dtype == torch.float32 else 5e-3), err
        assert (S[:2] == 1e4).all()                # other slots untouched


def _gates(H, T, i_scale, f_shift, seed=0):
    raw = _rand(T, 2 * H, dtype=torch.float32, seed=seed, scale=i_scale)
    raw[:, H:] += f_shift
    return raw


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("i_scale,f_shift", [(1.0, 3.0), (6.0, 6.0),
                                             (3.0, -8.0), (0.1, 12.0)])
@pytest.mark.parametrize("H,D,E", MEM)
def test_gated_memory(sv, H, D, E, i_scale, f_shift, dtype):
    T, cap = T_MEM, 5.0 if H == 3 else 15.0
    q, k, v, p = _mem_inputs(H, D, E, T, dtype, seed=9)
    raw = _gates(H, T, i_scale, f_shift, seed=H)
    raw[37] = 40.0                 # one input stands out and is carried on
    ib, fb = (_rand(H, dtype=dtype, seed=s) for s in (1, 2))
    x = raw.double()
    gi = cap * torch.tanh((x[:, :H] + ib.double()) / cap)
    gf = vo.log_sigmoid(cap * torch.tanh((x[:, H:] + fb.double()) / cap))
    f = lambda t, s: t.double().view(T, H, s)
    want, (S_w, n_w, m_w) = vo.gated_memory(f(q, D) * D ** -0.5, f(k, D),
                                            f(v, E), gi, gf)
    # o = S^T q / |n . q|: how far the division amplifies rounding
    cond, ns, ms = torch.zeros(T, H).double(), 0.0, torch.zeros(H).double()
    for t in range(T):
        mt = torch.maximum(gf[t] + ms, gi[t])
        ns = (torch.exp(gf[t] + ms - mt)[:, None] * ns
              + torch.exp(gi[t] - mt)[:, None] * f(k, D)[t])
        ms, qn = mt, f(q, D)[t] * D ** -0.5 * ns
        cond[t] = qn.abs().sum(1) / torch.maximum(
            qn.sum(1).abs(), torch.exp(-ms)) + 1.0
    want = want.reshape(T, H, E)
    nt = -(-E // 32)
    for cuts in CUTS:
        S = torch.full((2, H, D, E), -3e3).cuda()
        n = torch.full((2, H, nt, D), 9e3).cuda()
        m = torch.full((2, H, nt), 50.0).cuda()

        def gate(at, c):
            return sv.ExpGate(raw[at:at + c].cuda().contiguous(), ib.cuda(),
                              fb.cuda(), cap, D ** -0.5)

        got = _run_memory(sv, p, (H * D, H * D, H * E), cuts, H, gate, S, n,
                          m, slot=1)
        c = cond.unsqueeze(2)
        got = got.double().cpu().view(T, H, E)
        _close(want + (got - want) / c, want, torch.float32, 20.0,
               (H, D, E, cuts[:4])) if dtype == torch.float32 else \
            _close(got, want, dtype, 2.0, (H, D, E, cuts[:4]))
        assert (m[1].double().cpu() - m_w.view(H, 1)).abs().max() < 2e-3
        for got_s, w in ((S[1], S_w), (n[1], n_w.unsqueeze(1))):
            err = (got_s.double().cpu() - w).abs().max() / w.abs().max()
            assert err < 2e-4, err


@pytest.mark.parametrize("gated", [False, True])
@pytest.mark.parametrize("dtype", DTYPES)
def test_memory_batch_and_slots(sv, dtype, gated):
    """Segments of unequal length in one call equal each alone, whatever
    slots they use."""
    H, D, E = 2, 32, 48
    lens, slots = [70, 2, 529, 64], [3, 0, 4, 1]
    T = sum(lens)
    q, k, v, p = _mem_inputs(H, D, E, T, dtype, seed=11)
    raw = _gates(H, T, 1.0, 2.0).cuda()
    b = torch.zeros(H, dtype=dtype).cuda()
    mk = lambda: (torch.full((5, H, D, E), 5.0).cuda(),
                  torch.full((5, H, 2, D), 5.0).cuda(),
                  torch.full((5, H, 2), 5.0).cuda())

    def gate(a, e):
        if not gated:
            return sv.decay_gate([0.9, 0.99], "cuda")
        return sv.ExpGate(raw[a:e].contiguous(), b, b, 15.0, 0.2)

    starts = [sum(lens[:i]) for i in range(4)]
    pc = p.cuda()
    cut = lambda t: (t[:, :H * D], t[:, H * D:2 * H * D],
                     t[:, 2 * H * D:2 * H * D + H * E])
    seg, *tab = _tables(sv, [(s, a, n, 0) for s, a, n in
                             zip(slots, starts, lens)], True)
    S, n, m = mk()
    both = sv.memory_mix(*cut(pc), gate(0, T), S, n, m, seg, H, *tab)
    for s, a, ln in zip(slots, starts, lens):
        S1, n1, m1 = mk()
        one, *tab = _tables(sv, [(0, 0, ln, 0)], True)
        alone = sv.memory_mix(*cut(pc[a:a + ln]), gate(a, a + ln), S1, n1,
                              m1, one, H, *tab)
        assert torch.equal(alone, both[a:a + ln])
        assert torch.equal(S1[0], S[s])


# ---------------------------------------------------------------------------
# norms and pointwise steps
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [64, 100, 97, 1000, 4096])
def test_residual_norm(sv, W, dtype):
    T, eps = 9, 0.03
    x = _rand(T, W, dtype=torch.float32)
    a, b, x0 = (_rand(T, W, dtype=dtype, seed=s, scale=3.0)
                for s in (1, 2, 3))
    w, wa, wb, vec = (_rand(W, dtype=dtype, seed=s) for s in (4, 5, 6, 7))
    y = _rand(T, W, dtype=torch.float32, seed=8)
    d = lambda t: t.double()
    c = lambda t: t.cuda()
    cases = [
        (None, sv.Pending(c(a)), d(a)),
        (x, sv.Pending(c(a)), d(x) + d(a)),
        (x, None, d(x)),
        (None, sv.Pending(c(y), vec=c(vec)), d(y) + d(vec)),
        (x, sv.Pending(c(a), c(b), c(wa), c(wb), 0.5),
         d(x) + 0.5 * (vo.rms_norm(d(a), d(wa), eps)
                       + vo.rms_norm(d(b), d(wb), eps))),
    ]
    for res, pend, want in cases:
        r = None if res is None else res.cuda()
        nx, h, cat = sv.residual_norm(r, pend, eps, c(w), x0=c(x0))
        _close(nx, want, torch.float32)
        _close(h, vo.rms_norm(want, d(w), eps), dtype)
        _close(cat[:, :W], want, dtype)
        assert torch.equal(cat[:, W:].cpu(), x0)
        idx = torch.tensor([7, 0, 7], dtype=torch.int32).cuda()
        nx, h, _ = sv.residual_norm(r, pend, eps, c(w), keep_x=False,
                                    index=idx)
        assert nx is None
        _close(h, vo.rms_norm(want, d(w), eps)[[7, 0, 7]], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("groups,gs", [(1, 96), (3, 40), (2, 33), (1, 2048),
                                       (4, 1500), (5, 512)])
def test_gated_norm(sv, groups, gs, dtype):
    T, N, eps = 7, groups * gs, 0.02
    o = _rand(T, N, dtype=dtype)
    w = _rand(N, dtype=dtype, seed=1)
    fused = _rand(T, N + 24, dtype=dtype, seed=2)
    g = fused.cuda()[:, 24:]
    want = (vo.rms(o.double().view(T, groups, gs), eps).reshape(T, N)
            * w.double() * torch.sigmoid(fused[:, 24:].double()))
    _close(sv.gated_norm(o.cuda(), w.cuda(), g, gs, eps), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_pointwise(sv, dtype):
    x = _rand(13, 37, dtype=dtype, scale=4.0)
    _close(sv.relu_squared_(x.cuda()), vo.relu_squared(x.double()), dtype)
    y = _rand(5, 33, dtype=torch.float32, scale=60.0)
    _close(sv.softcap_(y.cuda(), 12.0),
           12.0 * torch.tanh(y.double() / 12.0), torch.float32)


def test_cpu_tensors_are_refused(sv):
    with pytest.raises(RuntimeError):
        sv.relu_squared_(torch.zeros(4, 4))
