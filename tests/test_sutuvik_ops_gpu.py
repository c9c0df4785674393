"""The kernels that Sutuvik added to the serving library, each against the
plain implementation: short convolutions and their rings, grouped norms,
prepared queries and keys, modified scores, timed memories, group-limited
routing."""

from types import SimpleNamespace

import pytest
import torch

import sutuvik_cases as sc
import sutuvik_oracle as so
from neuronx_distributed_amd.ops import serving as sv

pytestmark = pytest.mark.gpu

F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [F32, BF16]
TOL = {F32: 1e-5, BF16: 8e-3}


@pytest.fixture(scope="module", autouse=True)
def _built():
    sv.ensure_built()


def _rand(*shape, seed=0, dtype=F32):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(*shape, generator=g).to(dtype)


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device="cuda")


def _near(got, want, dtype, what="", tol=None):
    got, want = got.double().cpu(), want.double()
    assert got.shape == want.shape and torch.isfinite(got).all(), what
    err = (got - want).abs().max() / want.abs().max().clamp(min=1e-6)
    assert err < (tol or TOL[dtype]), (what, err.item())


def _segments(parts):
    """(slot, rows, context) of requests packed one after another -> the
    device tables of portions."""
    seg, at = [], 0
    for slot, rows, ctx in parts:
        seg.append((slot, at, rows, ctx))
        at += rows
    chunks, first = sv.chunk_table(seg)
    return _i32(seg), _i32(chunks), _i32(first)


# ---------------------------------------------------------------------------
# short convolutions
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6, 20, 65])
@pytest.mark.parametrize("C", [40, 13])
def test_short_conv_in_portions(dtype, taps, C):
    """Two requests in portions of several sizes on slots that held others:
    every cut gives the whole sequence's result."""
    T = 330
    x = _rand(2, T, C, seed=1, dtype=dtype)
    w = _rand(C, taps, seed=2, dtype=dtype)
    b = _rand(C, seed=3, dtype=dtype)
    want = [so.causal_conv(s.double(), w.double()) for s in x]
    ring = _rand(5, taps, C, seed=4, dtype=dtype).cuda() * 100
    conv = sv.ShortConv(w.t().contiguous().cuda(), ring, b.cuda())
    plain = sv.ShortConv(conv.w, ring)
    for cuts in ([T], [2] * 20 + [290], [1, 3, 64, 1, 261], [16, 16, 15, 283],
                 [256, 74], [2, 255, 73]):
        at = 0
        for n in cuts:
            seg, chunks, _ = _segments([(3, n, at), (1, n, at)])
            rows = x[:, at:at + n].reshape(2 * n, C).cuda()
            a = sv.short_conv(rows, conv, seg, chunks, silu=True)
            y = [v[at:at + n] for v in want]
            _near(a, torch.cat([so.silu(v + b.double()) for v in y]), dtype,
                  (cuts[:3], at))
            # the same once more: the ring's places are the same
            a = sv.short_conv(rows, plain, seg, chunks, add=True) \
                if n == T else None
            if a is not None:
                _near(a, torch.cat([v + s.double() for v, s in zip(y, x)]),
                      dtype, "add")
            at += n


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps,W,groups", [(4, 64, 2), (1, 48, 3), (7, 50, 5),
                                           (2, 4096, 8), (3, 60, 1)])
def test_norm_and_conv_of_mixed_rows(dtype, taps, W, groups):
    """residual_norm with a convolution: portions and single tokens of four
    requests in one batch, step after step."""
    eps, lens = 1e-4, [9, 70, 3, 300 if W < 100 else 40]
    xs = [_rand(n, W, seed=i) * torch.linspace(0.1, 3, W) for i, n in
          enumerate(lens)]
    w = _rand(W, seed=9, dtype=dtype)
    f = _rand(W, taps, seed=8, dtype=dtype)
    want = []
    for x in xs:
        h = so.group_norm(x.double(), w.double(), groups, eps)
        h = h.to(dtype).double()
        want.append(h + so.causal_conv(h, f.double()))
    ring = torch.full((6, taps, W), 50.0, dtype=dtype, device="cuda")
    conv = sv.ShortConv(f.t().contiguous().cuda(), ring)
    at, step = [0] * 4, 0
    while any(a < n for a, n in zip(at, lens)):
        step += 1
        take = [(i, min((1, 2, 1, 37)[(i + step) % 4], n - a))
                for i, (a, n) in enumerate(zip(at, lens)) if a < n]
        take.sort(key=lambda e: e[1] == 1)
        port = [(5 - i, n, at[i]) for i, n in take if n > 1]
        n = sum(p[1] for p in port)
        seg, chunks, _ = _segments(port) if port else (
            _i32([]).view(0, 4), _i32([]).view(0, 4), None)
        batch = SimpleNamespace(
            portion_tokens=n, portions=seg, chunks=chunks,
            singles=_i32([(5 - i, n + k, 1, at[i]) for k, (i, _) in
                          enumerate(e for e in take if e[1] == 1)]
                         ).view(-1, 4))
        rows = torch.cat([xs[i][at[i]:at[i] + m] for i, m in take])
        x_new, h, _ = sv.residual_norm(rows.cuda(), None, eps, w.cuda(),
                                       groups=groups, conv=conv, batch=batch,
                                       dtype=dtype)
        _near(h, torch.cat([want[i][at[i]:at[i] + m] for i, m in take]),
              dtype, step)
        _near(x_new, rows, F32)
        for i, m in take:
            at[i] += m


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,groups,p_groups", [(96, 3, 1), (96, 1, 4),
                                               (50, 5, 2), (2048, 64, 8),
                                               (64, 64, 64)])
def test_grouped_norms(dtype, W, groups, p_groups):
    """The pending result's norm and the output norm in groups, its scale."""
    x, d = _rand(7, W), _rand(7, W, seed=1, dtype=dtype) * torch.linspace(
        0.01, 4, W).to(dtype)
    w, w1 = _rand(W, seed=2, dtype=dtype), _rand(W, seed=3, dtype=dtype)
    want = x.double() + so.group_norm(d.double(), w1.double(), p_groups, 1e-3)
    x_new, h, _ = sv.residual_norm(
        x.cuda(), sv.Pending(d.cuda(), w1=w1.cuda(), groups=p_groups), 1e-3,
        w.cuda(), groups=groups, scale=0.37)
    _near(x_new, want, F32)
    _near(h, 0.37 * so.group_norm(want, w.double(), groups, 1e-3), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,group", [(96, 96), (96, 24), (50, 10),
                                     (2048, 2048)])
def test_norm_without_a_gate(dtype, N, group):
    x, w = _rand(5, N, dtype=dtype), _rand(N, seed=1, dtype=dtype)
    got = sv.gated_norm(x.cuda(), w.cuda(), None, group, 1e-2)
    _near(got, so.group_norm(x.double(), w.double(), N // group, 1e-2), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_token_gate(dtype):
    x, table = _rand(30, 9, dtype=dtype) * 2, _rand(12, 40, dtype=dtype)
    toks = torch.randint(0, 12, (30,))
    got = sv.gelu_rows_(x.cuda(), table.cuda(), toks.int().cuda(), 18)
    _near(got, so.gelu_tanh(x.double()) * table.double()[toks][:, 18:27],
          dtype)


# ---------------------------------------------------------------------------
# attention
# ---------------------------------------------------------------------------

def _pages(lens, G, D, E, dtype, spare=2):
    n = [-(-x // 64) for x in lens]
    ids = torch.randperm(sum(n) + spare,
                         generator=torch.Generator().manual_seed(5)).tolist()
    table, at = [], 0
    for k in n:
        table.append(ids[at:at + k] + [0] * (max(n) - k))
        at += k
    kc = torch.full((sum(n) + spare, G, 64, D), 30.0, dtype=dtype,
                    device="cuda")
    vc = torch.full((sum(n) + spare, G, 64, E), 30.0, dtype=dtype,
                    device="cuda")
    return kc, vc, _i32(table)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,E,dims,kind", [
    (4, 2, 56, 32, 16, "weighted"), (3, 1, 11, 10, 10, "weighted"),
    (2, 2, 128, 64, 128, "plain"), (2, 1, 200, 16, 64, "plain"),
    (5, 1, 40, 320, 0, None)])
def test_prepared_queries_and_keys(dtype, H, G, D, E, dims, kind):
    """Rotation at far positions, norm, temperature and mixed values: queries
    in place, keys and values in their pages."""
    T, eps = 20, 1e-3
    positions = [0, 1, 2, 6, 7, 8, 63, 64, 65, 127, 128, 200, 255, 256, 1000,
                 1001, 2047, 2048, 2999, 3000]
    rot = {"base": 500.0, "dims": dims, "scaling": {
        "factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}}
    q, k, v, first = (_rand(T, n * d, seed=i, dtype=dtype) for i, (n, d) in
                      enumerate(((H, D), (G, D), (G, E), (G, E))))
    qn, kn = (_rand(D, seed=i, dtype=dtype) for i in (7, 8))
    lam = torch.tensor(0.3, dtype=dtype)

    def made(x, n, w):
        x = x.double().view(T, n, D)
        if dims:
            x = so.rotate_pairs(x, positions, rot)
        if kind:
            x = so.rms(x, eps)
        return x * w.double() if kind == "weighted" else x

    wq, wk = made(q, H, qn), made(k, G, kn)
    wq = wq * torch.tensor([so.query_temperature(p, 0.4, 7)
                            for p in positions]).double().view(T, 1, 1)
    wv = so.mixed_values(v.double(), lam.double(), first.double())
    kc, vc, bt = _pages([3001], G, D, E, dtype)
    prep = sv.QkvPrep(
        freq=sv.rotary_frequencies(500.0, dims, "cuda", rot["scaling"])
        if dims else None, norm=kind is not None, eps=eps,
        q_norm=qn.cuda() if kind == "weighted" else None,
        k_norm=kn.cuda() if kind == "weighted" else None, temp_coef=0.4,
        temp_every=7, first=first.cuda(), mix=lam.cuda())
    pad = torch.cat([q, k, v], 1).cuda()
    q, k, v = pad.split([H * D, G * D, G * E], 1)
    sv.qkv_append(q, k, v, kc, vc, _i32(positions), _i32([0] * T), bt, H,
                  prep)
    _near(q, wq.reshape(T, H * D), dtype, "q")
    row = bt[0].tolist()
    at = [(row[p // 64], p % 64) for p in positions]
    _near(torch.stack([kc[a, :, b] for a, b in at]), wk, dtype, "k")
    _near(torch.stack([vc[a, :, b] for a, b in at]), wv.view(T, G, E), dtype,
          "v")
    left = torch.ones(kc.shape[0], 64, dtype=torch.bool)
    for a, b in at:
        left[a, b] = False
    assert (kc.cpu().transpose(1, 2)[left] == 30).all()   # and nothing else


MODS = {
    "bias": dict(slope=True, sink=True, gate=True),
    "cap": dict(cap=4.0, temp=True, sink=True),
    "all": dict(cap=6.0, temp=True, slope=True, sink=True, gate=True),
    "sink": dict(sink=True),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", list(MODS))
@pytest.mark.parametrize("H,G,D,E", [(4, 2, 56, 32), (3, 1, 11, 10),
                                     (8, 1, 128, 48), (2, 2, 64, 200),
                                     (6, 2, 160, 96)])
def test_modified_scores(dtype, kind, H, G, D, E):
    """Portions and decoded rows against the plain softmax; the first key, the
    keys at page borders and the newest stand out."""
    on, T = MODS[kind], 330
    q, k, v = sc.attention_case(T, H, G, D, E, 3, [0, 63, 64, 128, 255, 256])
    q, k, v = (x.to(dtype) for x in (q, k, v))
    scale = 3.0 * D ** -0.5
    temp = (1.0 + _rand(H, seed=1)).to(dtype) if on.get("temp") else None
    sink = (3.0 + 2 * _rand(H, seed=2)).to(dtype) if on.get("sink") else None
    gate = _rand(T, H, seed=4, dtype=dtype) if on.get("gate") else None
    cap, bias = on.get("cap", 0.0), on.get("slope", False)
    pos = torch.arange(T, dtype=torch.float64)
    want = []
    for h in range(H):
        s = q[:, h].double() @ k[:, h // (H // G)].double().T * scale
        if temp is not None:
            s = s * temp[h].double()
        if cap:
            s = cap * torch.tanh(s / cap)
        if bias:
            s = s - so.slope(h, H) * (pos[:, None] - pos[None])
        o = so.attend(s, v[:, h // (H // G)].double(), sink[h].double())
        if gate is not None:
            o = o * so.sigmoid(gate[:, h:h + 1].double())
        want.append(o)
    want = torch.cat(want, 1)
    slope = torch.tensor([so.slope(h, H) for h in range(H)]).float().cuda() \
        if bias else None
    mod = sv.ScoreMod(*(t.cuda() if t is not None else None
                        for t in (temp,)), cap=cap, slope=slope,
                      sink=sink.cuda(),
                      gate=gate.cuda() if gate is not None else None)
    kc, vc, bt = _pages([100, T], G, D, E, dtype)
    q, k, v = (x.reshape(T, -1).cuda() for x in (q, k, v))
    p32 = torch.arange(T, dtype=torch.int32, device="cuda")
    one = torch.ones(T, dtype=torch.int32, device="cuda")
    got, at = [], 0
    for n in (130, 2, 64, 134):
        r = slice(at, at + n)
        tiles = _i32([(1, s, min(128, n - s), at + s)
                      for s in range(0, n, 128)])
        got.append(sv.attn_portions(
            q[r], k[r], v[r], kc, vc, p32[r], one[r], bt, tiles, H, scale,
            mod=mod.rows(at, at + n), max_keys=T))
        at += n
    _near(torch.cat(got), want, dtype, "portions")
    for max_keys in (64, 2000):           # one and several workgroups a row
        r = slice(250, T)
        got = sv.attn_rows(q[r], k[r], v[r], kc, vc, p32[r], one[r], bt, H,
                           scale, append=False, max_keys=max_keys,
                           mod=mod.rows(250, T))
        _near(got, want[250:], dtype, "rows")
    r = slice(T - 1, T)                   # the row's own key from registers
    got = sv.attn_rows(q[r], k[r], v[r], kc, vc, p32[r], one[r], bt, H, scale,
                       max_keys=T, mod=mod.rows(T - 1, T))
    _near(got, want[r], dtype, "append")


def test_a_far_biased_key_is_not_lost():
    """A key thousands of positions back wins against its distance bias, in a
    prompt tile and when decoding."""
    dtype, T, D, far = BF16, 4200, 64, 70
    q = torch.zeros(T, 2, D)
    q[..., 0] = 1.0
    k, v = torch.zeros(T, 1, D), torch.zeros(T, 1, D)
    k[far, 0, 0], v[far, 0, 3] = 256.0, 1.0
    slope = torch.tensor([0.0625, 2.0 ** -8])
    mod = sv.ScoreMod(slope=slope.cuda(), sink=torch.full(
        (2,), 1.0, dtype=dtype).cuda())
    i = T - 1
    s = torch.zeros(2, T, dtype=torch.float64)
    s[:, far] = 256.0
    s = s - slope.double()[:, None] * (i - torch.arange(T).double())
    want = torch.exp(s[:, far]) / (torch.exp(s).sum(1) + torch.exp(
        torch.tensor(1.0).double()))
    kc, vc, bt = _pages([T], 1, D, D, dtype)
    q, k, v = (x.to(dtype).reshape(T, -1).cuda() for x in (q, k, v))
    p32 = torch.arange(T, dtype=torch.int32, device="cuda")
    zero = torch.zeros(T, dtype=torch.int32, device="cuda")
    tiles = _i32([(0, s, min(128, T - s), s) for s in range(0, T, 128)])
    a = sv.attn_portions(q, k, v, kc, vc, p32, zero, bt, tiles, 2, 1.0,
                         mod=mod)[i].view(2, D)[:, 3]
    b = sv.attn_rows(q[i:], k[i:], v[i:], kc, vc, p32[i:], zero[i:], bt, 2,
                     1.0, mod=mod, max_keys=T)[0].view(2, D)[:, 3]
    assert want[1] > 0.9
    _near(a, want, dtype)
    _near(b, want, dtype)


# ---------------------------------------------------------------------------
# timed memories
# ---------------------------------------------------------------------------

def _ssm(T, H, G, N, P, seed, dtype):
    x, B, C = (_rand(T, n, seed=seed + i, dtype=dtype)
               for i, n in enumerate((H * P, G * N, G * N)))
    z = _rand(T, H * P, seed=seed + 3, dtype=dtype)
    raw = 2.0 * _rand(T, H, seed=seed + 4)
    return x, B, C, z, raw


def _ssm_params(H, dtype):
    return ((_rand(H, seed=70) - 2).to(dtype),
            _rand(H, seed=71, dtype=dtype).clamp(-2, 2),
            _rand(H, seed=72, dtype=dtype))


def _ssm_want(case, params, H, G, N, P):
    x, B, C, z, raw = (t.double() for t in case)
    bias, A_log, skip = (t.double() for t in params)
    T = x.shape[0]
    dt = so.softplus(raw + bias)
    y, S = so.state_space(x.view(T, H, P), B.view(T, G, N), C.view(T, G, N),
                          dt, torch.exp(-torch.exp(A_log) * dt), skip)
    return y.reshape(T, H * P) * so.silu(z), S


SIZES = [(4, 2, 40, 56), (3, 1, 13, 7), (2, 1, 128, 64), (4, 1, 64, 136),
         (2, 2, 200, 16), (2, 1, 300, 40)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,N,P", SIZES)
def test_timed_memory(dtype, H, G, N, P):
    """Portions of several sizes, then single tokens, on a slot full of
    another request's state: outputs and the state."""
    T, n1 = 700, 640
    case, params = _ssm(T, H, G, N, P, 10, dtype), _ssm_params(H, dtype)
    want, S_want = _ssm_want(case, params, H, G, N, P)
    dev = [t.cuda() for t in case]
    pd = [t.cuda() for t in params]
    S = torch.full((3, H, N, P), 7.0, device="cuda")
    for cuts in ([n1], [2, 254, 256, 128], [300, 3, 337], [64] * 10):
        at, got = 0, []
        for n in cuts + [1] * (T - n1):
            x, B, C, z, raw = (t[at:at + n] for t in dev)
            gate = sv.TimeGate(raw, *pd, z)
            seg, chunks, first = _segments([(2, n, at)])
            tab = (chunks, first) if n > 1 else ()
            got.append(sv.memory_mix(C, B, x, gate, S, None, None, seg, H,
                                     *tab))
            at += n
        _near(torch.cat(got), want, dtype, cuts[:3])
        _near(S[2], S_want, F32, "state", 2e-5 if dtype == BF16 else 2e-6)
        assert (S[:2] == 7).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_timed_memory_in_batches(dtype):
    """Unequal portions of several requests in one call."""
    H, G, N, P = 4, 2, 64, 32
    lens, slots = [257, 2, 90, 512, 31], [4, 0, 3, 1, 2]
    cases = [_ssm(n, H, G, N, P, 20 * i, dtype) for i, n in enumerate(lens)]
    params = _ssm_params(H, dtype)
    x, B, C, z, raw = (torch.cat(t).cuda() for t in zip(*cases))
    S = torch.zeros(5, H, N, P, device="cuda")
    seg, chunks, first = _segments([(s, n, 0) for s, n in zip(slots, lens)])
    got = sv.memory_mix(C, B, x, sv.TimeGate(raw, *[t.cuda() for t in params],
                                             z), S, None, None, seg, H,
                        chunks, first)
    want = [_ssm_want(c, params, H, G, N, P) for c in cases]
    _near(got, torch.cat([w[0] for w in want]), dtype)
    for s, w in zip(slots, want):
        _near(S[s], w[1], F32, s, 2e-5 if dtype == BF16 else 2e-6)


@pytest.mark.parametrize("dtype", DTYPES)
def test_an_old_input_is_still_in_the_state(dtype):
    """Decays near one: an input 2000 tokens back decides the output."""
    H, G, N, P, T = 1, 1, 32, 32, 2050
    x, B, C = torch.zeros(T, P), torch.zeros(T, N), torch.zeros(T, N)
    x[3, 5], B[3, 2] = 1.0, 1.0
    C[:, 2] = 1.0
    z = torch.full((T, P), 1.0)
    raw = torch.full((T, H), -7.0)
    raw[3] = 1.0
    case = [t.to(dtype) for t in (x, B, C, z)] + [raw]
    params = (torch.zeros(H).to(dtype), torch.zeros(H).to(dtype),
              torch.zeros(H).to(dtype))
    want, _ = _ssm_want(case, params, H, G, N, P)
    assert want[-1, 5] > 0.01
    S = torch.zeros(1, H, N, P, device="cuda")
    dev, pd = [t.cuda() for t in case], [t.cuda() for t in params]
    got, at = [], 0
    for n in (1000, 1049, 1):
        a, b, c, zz, r = (t[at:at + n] for t in dev)
        seg, chunks, first = _segments([(0, n, at)])
        got.append(sv.memory_mix(c, b, a, sv.TimeGate(r, *pd, zz), S, None,
                                 None, seg, H,
                                 *((chunks, first) if n > 1 else ())))
        at += n
    _near(torch.cat(got)[:, 5], want[:, 5], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 4, 9])
@pytest.mark.parametrize("H,G,N,P", [(4, 2, 40, 56), (3, 1, 13, 7),
                                     (4, 4, 136, 40)])
def test_convolution_fused_into_single_tokens(dtype, taps, H, G, N, P):
    """Decoding from the first token, and after a portion, with q, k and v
    that have not passed their convolution."""
    T, inner, gn = 40, H * P, G * N
    C = inner + 2 * gn
    raw_x = _rand(T, C, seed=1, dtype=dtype)
    w, b = _rand(C, taps, seed=2, dtype=dtype) * 0.5, _rand(C, seed=3,
                                                           dtype=dtype)
    z, step = _rand(T, inner, seed=4, dtype=dtype), _rand(T, H, seed=5)
    params = _ssm_params(H, dtype)
    y = so.silu(so.causal_conv(raw_x.double(), w.double()) + b.double())
    x, B, Cm = y.split([inner, gn, gn], 1)
    want, _ = _ssm_want((x, B, Cm, z, step), params, H, G, N, P)
    pd = [t.cuda() for t in params]
    proj = torch.cat([z, raw_x], 1).cuda()
    step = step.cuda()
    for start in (0, 1, 17):
        S = torch.full((2, H, N, P), 3.0, device="cuda")
        ring = torch.full((2, taps, C), 9.0, dtype=dtype, device="cuda")
        conv = sv.ShortConv(w.t().contiguous().cuda(), ring, b.cuda())
        got = []
        if start:
            seg, chunks, first = _segments([(1, start, 0)])
            r = slice(0, start)
            a = sv.short_conv(proj[r, inner:], conv, seg, chunks, silu=True)
            a = a.split([inner, gn, gn], 1)
            got.append(sv.memory_mix(a[2], a[1], a[0], sv.TimeGate(
                step[r], *pd, proj[r, :inner]), S, None, None, seg, H, chunks,
                first))
        for t in range(start, T):
            r = slice(t, t + 1)
            a = proj[r, inner:].split([inner, gn, gn], 1)
            got.append(sv.memory_mix(
                a[2], a[1], a[0], sv.TimeGate(step[r], *pd, proj[r, :inner],
                                              conv), S, None, None,
                _i32([(1, 0, 1, t)]), H))
        _near(torch.cat(got), want, dtype, start, 2e-2 if dtype == BF16
              else 4e-6)


# ---------------------------------------------------------------------------
# routing
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("T", [1, 30, 200])
@pytest.mark.parametrize("E,top,groups,keep", [
    (14, 2, 2, 1), (20, 3, 4, 3), (7, 2, 7, 3), (9, 4, 1, 1), (64, 6, 8, 4),
    (256, 8, 8, 4), (512, 10, 64, 5), (6, 6, 2, 2)])
def test_group_limited_routing(T, E, top, groups, keep):
    """Chosen experts and weights; corrections push choice scores below zero,
    so a dropped group may not count as zero."""
    z = _rand(T, E, seed=E + T)
    bias = _rand(E, seed=4, dtype=BF16) - 1.5
    idx, w = so.route(z.double(), bias.double(), groups, keep, top)
    p = sv.moe_plan(z.cuda(), bias.cuda(), sv.Routing(top, True, groups, keep),
                    0)
    assert torch.equal(p.idx.cpu().long(), idx)
    _near(p.coef, w, F32, tol=1e-5)
    order = p.order.cpu().long()
    assert torch.equal(order.sort().values, torch.arange(T * top))
    assert (idx.flatten()[order].diff() >= 0).all()


def test_equal_scores_take_the_lower_index():
    z = torch.zeros(3, 8)
    p = sv.moe_plan(z.cuda(), None, sv.Routing(3, True, 4, 2), 0)
    assert p.idx.tolist() == [[0, 1, 2]] * 3
    _near(p.coef, torch.full((3, 3), 1 / 3), F32)


def test_bad_arguments_are_refused():
    z = torch.randn(4, 8).cuda()
    for r in (sv.Routing(3, True, 4, 1), sv.Routing(2, True, 3, 1),
              sv.Routing(2, True, 4, 5), sv.Routing(9, True)):
        with pytest.raises(ValueError):
            sv.moe_plan(z, None, r, 0)
    with pytest.raises(RuntimeError):
        sv.gelu_rows_(torch.zeros(2, 4), torch.zeros(3, 8),
                      torch.zeros(2, dtype=torch.int32), 0)
