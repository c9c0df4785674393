"""Latent attention, mixture of experts and output norms on the GPU, each
against the plain implementation in ``nesilorn_oracle`` (float64), one
mechanism at a time."""

import pytest
import torch

import nesilorn_oracle as no

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


def _ints(x):
    return torch.tensor(x, dtype=torch.int32).cuda()


class Batch:
    """The fields of a step that latent attention reads: portions first."""

    def __init__(self, sv, parts, bt, window, expand):
        """parts: (request, context, rows) with portions first."""
        pos, seq, tiles, segs = [], [], [], []
        for r, ctx, n in parts:
            if n > 1:
                tiles += [(len(segs), len(pos) + s, min(128, n - s), ctx + s)
                          for s in range(0, n, 128)]
                segs.append((r, len(pos), n, ctx))
            seq += [r] * n
            pos += range(ctx, ctx + n)
        self.pos, self.seq, self.block_table = _ints(pos), _ints(seq), bt
        self.portion_tokens = sum(n for _, _, n in parts if n > 1)
        self.max_keys = max(pos) + 1
        self.tiles = _ints(tiles) if tiles else None
        self.spans = {}
        if segs and expand:
            rows = [bt[r].tolist() for r, _, _, _ in segs]
            pages, table = sv.key_spans(segs, rows, window)
            self.spans = {window: sv.KeySpans(_ints(pages), _ints(table))}


def _cache(lengths, width, dtype, seed=0):
    """Scattered pages full of large stale values, and their table."""
    g = torch.Generator().manual_seed(seed)
    per = [-(-n // 64) for n in lengths]
    perm = torch.randperm(sum(per) + 2, generator=g).int()
    bt = torch.full((len(lengths), max(per) + 1), int(perm[-1]),
                    dtype=torch.int32)
    at = 0
    for r, n in enumerate(per):
        bt[r, :n] = perm[at:at + n]
        at += n
    return torch.full((sum(per) + 2, 64, width), 77.0, dtype=dtype).cuda(), \
        bt.cuda()


# H, dim, rot, vdim, rank, window
LATENT = [
    (4, 32, 16, 24, 48, 90),
    (3, 24, 8, 40, 72, 33),
    (36, 16, 16, 16, 136, 64),      # more than 32 heads
    (2, 128, 64, 128, 512, 130),
    (5, 64, 32, 64, 256, 0),        # plain causal
    (33, 8, 64, 8, 320, 1),
    (3, 10, 6, 7, 21, 70),          # sizes that are no multiple of 8
    (2, 40, 80, 200, 600, 65),      # too large for the MFMA row kernel
    (2, 112, 48, 96, 64, 90),       # key and value tiles with empty columns
    (2, 6, 2, 3, 9, 0),             # odd sums from several key ranges
]


def _latent_case(sv, H, D, P, E, R, window, T, dtype, seed=0, base=300.0):
    q = _rand(T, H * (D + P), dtype=dtype, seed=seed)
    kv = _rand(T, R + P, dtype=dtype, seed=seed + 1)
    gate = _rand(T, H * E, dtype=dtype, seed=seed + 2)
    norm = (1 + _rand(R, dtype=torch.float32, seed=5, scale=0.2)).to(dtype)
    uk = _rand(H * D, R, dtype=dtype, seed=6, scale=R ** -0.5)
    uv = _rand(H * E, R, dtype=dtype, seed=7, scale=R ** -0.5)
    w = sv.LatentWeights(
        norm.cuda(), uk.view(H, D, R).transpose(1, 2).contiguous().cuda(),
        torch.cat([uk, uv]).cuda(), sv.rotary_frequencies(base, P, "cuda"))
    cfg = {"heads": H, "dim": D, "rot_dim": P, "vdim": E, "kv_rank": R,
           "scale": 1.7 * (D + P) ** -0.5, "rot": {"base": base, "dims": P},
           "mask": {"size": window} if window else None}
    d = torch.float64
    c, kr = no.latents(kv.to(d), norm.to(d), R, base, range(T), 1e-5)
    want = no.latent_attention(q.to(d), c, kr, uk.to(d), uv.to(d), cfg,
                               range(T)) * no.sigmoid(gate.to(d))
    return q, kv, gate, w, cfg, want


def _run(sv, b, q, kv, gate, cache, w, cfg):
    return sv.latent_attention(
        q.cuda(), kv.cuda(), gate.cuda(), b, cache, w, cfg["heads"],
        cfg["dim"], cfg["vdim"], cfg["scale"], 1e-5,
        (cfg["mask"] or {}).get("size", 0))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", LATENT)
def test_latent_attention_portions_and_decoding(sv, case, dtype):
    H, D, P, E, R, window = case
    T = 210
    q, kv, gate, w, cfg, want = _latent_case(sv, *case, T, dtype)
    for expand in (True, False):
        for cuts in ([T], [2, 62, 64, 3, 50, 29], [130] + [1] * 80,
                     [1, 1, 2, 1, 63, 2, 140]):
            cache, bt = _cache([T], R + P, dtype, seed=len(cuts))
            out, at = [], 0
            for n in cuts:
                s = slice(at, at + n)
                b = Batch(sv, [(0, at, n)], bt, window, expand)
                out.append(_run(sv, b, q[s], kv[s], gate[s], cache, w, cfg))
                at += n
            _close(torch.cat(out), want, dtype, 4.0, (case, expand, cuts[:4]))


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_mixed_batch(sv, dtype):
    """Portions of two requests beside single tokens of two others."""
    case = (5, 32, 16, 40, 64, 70)
    ctx, rows = [100, 0, 130, 63], [70, 33, 1, 1]
    cases = [_latent_case(sv, *case, c + n, dtype, seed=10 * i)
             for i, (c, n) in enumerate(zip(ctx, rows))]
    w, cfg = cases[0][3], cases[0][4]
    for expand in (True, False):
        cache, bt = _cache([c + n for c, n in zip(ctx, rows)], 80, dtype)
        for i, c in enumerate(ctx):
            if c:
                q, kv, g = cases[i][:3]
                b = Batch(sv, [(i, 0, c)], bt, 70, expand)
                _run(sv, b, q[:c], kv[:c], g[:c], cache, w, cfg)
        b = Batch(sv, [(i, c, n) for i, (c, n) in enumerate(zip(ctx, rows))],
                  bt, 70, expand)
        q, kv, g = (torch.cat([cases[i][k][c:] for i, c in enumerate(ctx)])
                    for k in range(3))
        got = _run(sv, b, q, kv, g, cache, w, cfg)
        _close(got, torch.cat([cases[i][5][c:] for i, c in enumerate(ctx)]),
               dtype, 4.0, expand)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window", [64, 70, 33, 128, 1, 65])
def test_latent_window_edges_show(sv, window, dtype):
    """One key stands out; queries just inside see it, just outside do not.
    Rows of a cache that is written here, queries that meet one latent."""
    H, D, P, E, R, T = 3, 16, 8, 24, 40, 330
    d = torch.float64
    uk = torch.zeros(H * D, R)
    uk[::D, 0] = 1.0                        # first dim of a key = latent 0
    uv = _rand(H * E, R, dtype=dtype, scale=R ** -0.5, seed=3).float()
    uv[:, 0] = 0
    w = sv.LatentWeights(
        torch.ones(R, dtype=dtype).cuda(), uk.view(H, D, R).transpose(1, 2)
        .contiguous().to(dtype).cuda(), torch.cat([uk, uv]).to(dtype).cuda(),
        sv.rotary_frequencies(100.0, P, "cuda"))
    for spot in (0, 1, 63, 64, 65, 127, 128, 200):
        rows = _rand(T, R + P, dtype=dtype, seed=4)
        rows[:, 0] = 0.0
        rows[spot, 0] = 14.0
        rows[spot, 1:R] = 6.0
        q = _rand(T, H * (D + P), dtype=dtype, seed=5, scale=0.3)
        q[:, ::D + P] = 8.0
        qd = q.to(d).view(T, H, D + P)
        k = torch.cat([(rows[:, :R].to(d) @ uk.to(d).T).view(T, H, D),
                       rows[:, R:].to(d).view(T, 1, P).expand(T, H, P)], -1)
        v = (rows[:, :R].to(d) @ uv.to(dtype).to(d).T).view(T, H, E)
        want = no.window_attention(qd, k, v, 0.11, window).view(T, H * E)
        cache, bt = _cache([T], R + P, dtype, seed=spot)
        for p in range(-(-T // 64)):
            part = rows[64 * p:64 * p + 64].cuda()
            cache[int(bt[0, p]), :len(part)] = part
        places = sorted({p for p in (spot - 1, spot, spot + 1,
                                     spot + window - 1, spot + window,
                                     spot + window + 1, T - 1)
                         if 0 <= p < T})
        # as single tokens
        ql = torch.empty(len(places), H * (R + P), dtype=dtype).cuda()
        qs = q[places].cuda()
        ql.view(-1, H, R + P)[..., R:] = qs.view(-1, H, D + P)[..., D:]
        sv.head_linear(qs, D + P, w.absorb, ql, R + P)
        lat = sv.latent_rows(ql, cache, R, _ints(places),
                             _ints([0] * len(places)), bt, H, 0.11, window,
                             T)
        out = torch.empty(len(places), H * E, dtype=dtype).cuda()
        sv.head_linear(lat, R, w.expand[H * D:].view(H, E, R), out, E)
        _close(out, want[places], dtype, 3.0, (window, spot, "rows"))
        if dtype == torch.float32:
            continue
        for a, n in ((0, T), (spot + window - 2, 4), (spot, 2), (65, 200)):
            a, n = max(0, a), min(n, T - max(0, a))
            if n < 1:
                continue
            b = Batch(sv, [(0, a, n)], bt, window, True)
            if n == 1:
                continue
            out = torch.empty(n, H * E, dtype=dtype).cuda()
            sv.latent_portions(q[a:a + n].cuda(), None, cache, w, b,
                               b.spans[window], H, D, E, 0.11, window, out)
            _close(out, want[a:a + n], dtype, 3.0, (window, spot, a, n))


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_far_out_and_partial(sv, dtype):
    """Angles stay exact at large positions; columns past the rotated ones
    pass through; the latent is normed."""
    H, D, P, R, rot, base = 2, 6, 12, 20, 8, 10000.0
    where = [0, 1, 63, 64, 5000, 131071]
    T = len(where)
    q = _rand(T, H * (D + P), dtype=dtype)
    kv = _rand(T, R + P, dtype=dtype, seed=3)
    norm = _rand(R, dtype=dtype, seed=4)
    cache = torch.zeros(T, 64, R + P, dtype=dtype).cuda()
    bt = torch.zeros(T, 131072 // 64, dtype=torch.int32)
    for t, p in enumerate(where):
        bt[t, p // 64] = t
    w = sv.LatentWeights(norm.cuda(), None, None,
                         sv.rotary_frequencies(base, rot, "cuda"))
    qr = torch.zeros(T, H * (R + P), dtype=dtype).cuda()
    qc = q.cuda()
    args = (kv.cuda(), w, cache, _ints(where), _ints(list(range(T))),
            bt.cuda(), H, 1e-3)
    sv.latent_append(qc, D, D + P, qr, R, R + P, *args)
    assert torch.equal(qc.cpu(), q)
    sv.latent_append(qc, D, D + P, qc, D, D + P, *args)

    def turned(x):
        x = x.double()
        return torch.cat([no.rotate(x[..., :rot], where, base),
                          x[..., rot:]], -1)

    want = turned(q.view(T, H, D + P)[..., D:])
    _close(qr.view(T, H, R + P)[..., R:], want, dtype, what="q elsewhere")
    _close(qc.view(T, H, D + P)[..., D:], want, dtype, what="q in place")
    assert torch.equal(qc.cpu().view(T, H, D + P)[..., :D],
                       q.view(T, H, D + P)[..., :D])
    rows = torch.stack([cache[t, p % 64] for t, p in enumerate(where)])
    _close(rows[:, :R], no.plain_norm(kv[:, :R].double(), norm.double(),
                                      1e-3), dtype, what="latent")
    _close(rows[:, R:], turned(kv[:, R:]), dtype, what="shared key")
    assert int((cache != 0).any(-1).sum()) == T      # and nothing else


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,N,K,T", [(3, 48, 24, 5), (2, 512, 128, 33),
                                     (5, 128, 512, 70), (1, 20, 264, 1),
                                     (4, 7, 13, 3), (2, 36, 8, 2)])
def test_head_linear(sv, H, N, K, T, dtype):
    x = _rand(T, H * (K + 8), dtype=dtype)
    w = _rand(H, N, K, dtype=dtype, seed=1, scale=K ** -0.5)
    gate = _rand(T, H * N, dtype=dtype, seed=2)
    for g in (None, gate):
        out = torch.full((T, H * (N + 16)), 3.0, dtype=dtype).cuda()
        sv.head_linear(x.cuda(), K + 8, w.cuda(), out, N + 16,
                       None if g is None else g.cuda())
        got = out.view(T, H, N + 16)
        want = torch.stack([x.double().view(T, H, K + 8)[:, h, :K]
                            @ w[h].double().T for h in range(H)], 1)
        if g is not None:
            want = want * no.sigmoid(g.double()).view(T, H, N)
        _close(got[..., :N].reshape(T, -1), want.reshape(T, -1), dtype)
        assert (got[..., N:] == 3.0).all()


# ---------------------------------------------------------------------------
# mixture of experts
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("T,E,top", [(1, 3, 1), (5, 8, 8), (64, 65, 6),
                                     (65, 130, 4), (300, 512, 20),
                                     (700, 8, 2)])
@pytest.mark.parametrize("how", [0, 3, 4, 5])
def test_plan_routes_and_groups(sv, T, E, top, how):
    z = _rand(T, E, dtype=torch.float32)
    bias = _rand(E, dtype=torch.float32, seed=1)
    p = sv.moe_plan(z.cuda(), bias.cuda(), top, how)
    idx, w = no.route(z.double() + bias.double(), top)
    assert torch.equal(p.idx.cpu().long(), idx)
    _close(p.coef, w, torch.float32)
    order, tiles = p.order.cpu().tolist(), p.tiles.cpu().tolist()
    assert sorted(order) == list(range(T * top))
    flat, seen = idx.reshape(-1).tolist(), []
    for e, s0, n, _ in tiles:
        assert 0 <= n <= sv.MOE_TILE_ROWS[how]
        if n:
            assert all(flat[q] == e for q in order[s0:s0 + n])
            seen += range(s0, s0 + n)
    assert seen == list(range(T * top))


def test_kernel_of_the_grouped_products_fits_the_load():
    from neuronx_distributed_amd.ops import serving as sv

    rows = [sv.MOE_TILE_ROWS[sv.moe_kernel(n, 8)]
            for n in (1, 40, 64, 300, 1000, 5000)]
    assert rows == [32, 32, 32, 64, 128, 256]


def test_plan_breaks_ties_by_index_and_takes_uneven_loads(sv):
    z = torch.zeros(70, 9)
    p = sv.moe_plan(z.cuda(), None, 3, 0)
    assert (p.idx.cpu() == torch.tensor([0, 1, 2])).all()
    _close(p.coef, torch.full((70, 3), 1 / 3), torch.float32)
    z[:, 7] = 5.0                  # every row to one expert
    p = sv.moe_plan(z.cuda(), None, 1, 4)
    assert (p.idx.cpu() == 7).all()
    assert [t[:3] for t in p.tiles.cpu().tolist() if t[2]] == [[7, 0, 70]]


EXPERTS = [
    # T, experts, top, width, ff, limit
    (1, 4, 2, 64, 40, 0.8),
    (7, 8, 4, 96, 72, 1.5),
    (40, 5, 2, 136, 264, 0.7),
    (300, 6, 3, 256, 176, 2.0),
    (260, 16, 1, 640, 136, 1.0),
    (33, 3, 2, 50, 27, 0.9),       # sizes that are no multiple of 8
    (129, 4, 4, 512, 320, 7.0),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", EXPERTS)
def test_experts(sv, case, dtype):
    T, E, top, W, ff, limit = case
    h = _rand(T, W, dtype=dtype)
    z = _rand(T, E, dtype=torch.float32, seed=1)
    bias = _rand(E, dtype=dtype, seed=2)
    gate = _rand(E, ff, W, dtype=dtype, seed=3, scale=1.5 * W ** -0.5)
    up = _rand(E, ff, W, dtype=dtype, seed=4, scale=1.5 * W ** -0.5)
    down = _rand(E, W, ff, dtype=dtype, seed=5, scale=ff ** -0.5)
    idx, w = no.route(z.double() + bias.double(), top)
    want = torch.zeros(T, W, dtype=torch.float64)
    d = torch.float64
    for e in range(E):
        y = no.clamped_glu(h.to(d) @ gate[e].to(d).T,
                           h.to(d) @ up[e].to(d).T, limit) @ down[e].to(d).T
        want += y * (w * (idx == e)).sum(1, keepdim=True)
    gu = torch.cat([gate, up], 1).cuda()
    hows = [sv.MOE_PLAIN]
    if dtype == torch.bfloat16 and W % 8 == 0 and ff % 8 == 0:
        hows += [sv.MOE_STREAM, *sv.MOE_TILES]
    for how in hows:
        p = sv.moe_plan(z.cuda(), bias.cuda(), top, how)
        act = sv.moe_gemm(h.cuda(), gu, p, True, 1.702, limit, 1.0)
        y = sv.moe_gemm(act, down.cuda(), p, False)
        x, _, _ = sv.residual_norm(None, sv.Pending(y, coef=p.coef), 1e-5,
                                   copy=True, dtype=dtype)
        _close(x, want, dtype, 2.0, (case, how))
    pend = sv.moe_mlp(h.cuda(), z.cuda(), bias.cuda(), gu, down.cuda(), top,
                      1.702, limit, 1.0)
    x, _, _ = sv.residual_norm(None, pend, 1e-5, copy=True, dtype=dtype)
    _close(x, want, dtype, 2.0, case)


def test_plain_swiglu_is_the_default_activation(sv):
    T, E, W, ff, dtype = 9, 2, 64, 32, torch.float32
    h = _rand(T, W, dtype=dtype)
    gu = _rand(E, 2 * ff, W, dtype=dtype, scale=0.3)
    p = sv.moe_plan(_rand(T, E, dtype=dtype).cuda(), None, 2, sv.MOE_PLAIN)
    act = sv.moe_gemm(h.cuda(), gu.cuda(), p, True).cpu().double()
    idx = p.idx.cpu().reshape(-1)
    for slot, pair in enumerate(p.order.tolist()):
        y = gu[idx[pair]].double() @ h[pair // 2].double()
        _close(act[slot], y[:ff] * no.sigmoid(y[:ff]) * y[ff:], dtype)


# ---------------------------------------------------------------------------
# norms and pointwise
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,W,parts", [(3, 50, 1), (5, 128, 4),
                                          (70, 264, 2), (2, 4096, 3)])
def test_output_norms(sv, rows, W, parts, dtype):
    """x + norm(pending), its rounding, and the final norm of chosen rows."""
    x = _rand(rows, W, dtype=torch.float32)
    w1 = _rand(W, dtype=dtype, seed=1, scale=0.3)
    w2 = _rand(W, dtype=dtype, seed=2, scale=0.3)
    y = _rand(rows * parts, W, dtype=dtype, seed=3)
    coef = torch.rand(rows, parts)
    d = torch.float64
    plain = y.to(d).view(rows, parts, W)
    pick = torch.tensor([rows - 1, 0, rows - 1], dtype=torch.int32)
    for mixed in (False, True):
        if mixed:
            src = (plain * coef.to(d)[..., None]).sum(1)
            pend = lambda **k: sv.Pending(y.cuda(), coef=coef.cuda(), **k)
        else:
            src = plain[:, 0]
            pend = lambda **k: sv.Pending(
                y.view(rows, parts, W)[:, 0].contiguous().cuda(), **k)
        for centred in (False, True):
            for scale in (1.0, 0.3):
                nw = (1.0 if centred else 0.0) + w1.to(d)
                for normed in (False, True):
                    kw = dict(centred=centred, scale=scale)
                    if normed:
                        kw["w1"] = w1.cuda()
                    add = no.rms(src, 1e-3) * nw if normed else src
                    for base in (x, None):
                        new = scale * add + (0 if base is None else x.to(d))
                        b = None if base is None else x.cuda()
                        xs, h, _ = sv.residual_norm(b, pend(**kw), 1e-3,
                                                    copy=True, dtype=dtype)
                        _close(xs, new, torch.float32, 2.0)
                        _close(h, new, dtype)
                        fw = (1.0 if centred else 0.0) + w2.to(d)
                        none, h, _ = sv.residual_norm(
                            b, pend(**kw), 1e-3, w2.cuda(), keep_x=False,
                            index=pick.cuda(), centred=centred)
                        assert none is None
                        _close(h, (no.rms(new, 1e-3) * fw)[pick.long()],
                               dtype, 1.5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 77, 4096])
def test_gelu(sv, n, dtype):
    x = (_rand(n, dtype=torch.float32) * 4).to(dtype)
    x[0] = -30.0
    want = no.gelu_tanh(x.double())
    got = sv.gelu_tanh_(x.cuda()).double().cpu()
    tol = 1e-6 if dtype == torch.float32 else 5e-3
    assert ((got - want).abs() <= tol * want.abs().clamp(min=1.0)).all()


def test_kernels_refuse_the_cpu(sv):
    x = torch.randn(4, 8)
    with pytest.raises(RuntimeError):
        sv.gelu_tanh_(x)
    with pytest.raises(RuntimeError):
        sv.head_linear(x, 8, torch.randn(1, 8, 8), torch.empty(4, 8), 8)
    with pytest.raises(ValueError):
        sv.moe_plan(torch.randn(4, 8).cuda(), None, 9, 0)
