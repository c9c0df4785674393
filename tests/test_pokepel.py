"""What of the Pokepel design needs no GPU: configuration, weights, state
specifications; and the oracle's own forms and its sensitivity to planted
mistakes."""

import json
import math

import pytest
import torch

import pokepel_cases as pc
import pokepel_oracle as po
from neuronx_distributed_amd.inference import (CacheManager, MatrixState,
                                               PagedLatent)
from neuronx_distributed_amd.ops import serving as sv


@pytest.fixture
def groups():
    from neuronx_distributed_amd.inference import single_process_groups

    single_process_groups()


# ---------------------------------------------------------------------------
# registry, configuration, weights, state
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("case", list(pc.CASES))
def test_load_pretrained_by_config(case, tmp_path, groups):
    from neuronx_distributed_amd.models import (PokepelForCausalLM,
                                                load_pretrained)

    cfg = pc.CASES[case]
    w = pc.weights(cfg)
    pc.save(cfg, w, tmp_path)
    m = load_pretrained(str(tmp_path), torch.float32)
    assert isinstance(m, PokepelForCausalLM)
    assert {p.dtype for p in m.parameters()} == {torch.float32}
    assert torch.equal(m.head, w["head"].float())
    for i, (L, layer) in enumerate(zip(cfg["layers"], m.layers)):
        p, c, f = f"l{i}.", L["mixer"], L["mlp"]
        block, mix = layer.block, layer.block.mixer
        names = ("q", "k", "v", "g") if L["type"] == "retention" else \
            ("q", "dkv", "g")
        parts = [[w[f"{p}mix.{n}"] for n in names], [w[p + "rg1"]]]
        if f is not None:
            inp = ["up"] if f["kind"] == "dense" else ["shared.gate",
                                                       "shared.up"]
            parts += [[w[f"{p}mlp.{n}"] for n in inp], [w[p + "rg2"]]]
            assert torch.equal(block.bias2, w[p + "rg2.b"].float())
        else:
            assert block.mlp is None and not hasattr(block, "bias2")
        assert torch.equal(block.bias1, w[p + "rg1.b"].float())
        rest = torch.ones(block.proj.weight.shape[0], dtype=torch.bool)
        assert len(parts) == len(block.at)
        for (a, b), part in zip(block.at, parts):
            assert a % 8 == 0 and torch.equal(block.proj.weight[a:b],
                                              torch.cat(part).float())
            rest[a:b] = False
        assert not block.proj.weight[rest].any()
        H = c["heads"]
        if L["type"] == "retention":
            assert layer.cache_specs() == [
                MatrixState(H, c["dim"], c["vdim"])]
            assert mix.decay == c["decay"] and mix.norm is None
        else:
            assert layer.cache_specs() == [
                PagedLatent(c["kv_rank"], c["rot_dim"])]
            assert torch.equal(mix.sink, w[p + "mix.sink"].float())
            assert torch.equal(mix.expand[:H * c["dim"]],
                               w[p + "mix.uk"].float())
        if f is None:
            continue
        if f["kind"] == "dense":
            assert torch.equal(block.mlp.act, w[p + "mlp.act"].float())
            continue
        r, ff = f["router"], f["expert"]["ff"]
        ex = block.mlp.experts
        assert ex.bias is None and ex.routing == sv.Routing(
            r["top"], False, r["groups"]["count"], r["groups"]["keep"], True,
            1)
        for e in range(r["experts"]):
            q = f"{p}mlp.e{e}."
            assert torch.equal(ex.gate_up[e], torch.cat(
                [w[q + "gate"], w[q + "up"]]).float())
            assert torch.equal(ex.down[e], w[q + "down"].float())
        assert torch.equal(block.mlp.down.weight,
                           w[p + "mlp.shared.down"].float())


def test_experts_without_a_shared_one(groups):
    from neuronx_distributed_amd.models import PokepelConfig, build_model

    cfg = json.loads(json.dumps(pc.CASES["memories"]))
    w = {k: v for k, v in pc.weights(cfg).items() if ".shared." not in k}
    cfg["layers"][0]["mlp"]["shared"] = None
    m = build_model("Pokepel", PokepelConfig.from_dict(cfg), torch.float32)
    m.load_checkpoint(w)
    a, b = m.layers[0].block.at[2]
    assert a == b


def test_bad_checkpoints_are_refused(groups):
    from neuronx_distributed_amd.models import PokepelConfig, build_model

    cfg = pc.CASES["odd"]
    w = pc.weights(cfg)
    m = build_model("Pokepel", PokepelConfig.from_dict(cfg), torch.float32)
    m.load_checkpoint(w)
    # gates of a feed-forward that is not there have no place, and do no harm
    m.load_checkpoint({**w, "l4.rg2": w["l3.rg2"], "l4.rg2.b": w["l3.rg2.b"]})
    for name in ("l0.mix.sink", "l1.mlp.act", "l2.rg2.b", "head",
                 "l3.mlp.shared.up", "l0.norm1"):
        with pytest.raises(KeyError):
            m.load_checkpoint({k: v for k, v in w.items() if k != name})
    with pytest.raises(KeyError):
        m.load_checkpoint({**w, "l0.norm2": w["l0.norm1"]})
    for name in ("embed", "head", "l0.mix.q", "l1.mix.k", "l0.mix.dkv",
                 "l0.mix.uk", "l2.mix.sink", "l1.mlp.act", "l1.mlp.up",
                 "l0.rg1", "l0.rg2.b", "l0.mlp.router",
                 "l0.mlp.shared.gate"):
        with pytest.raises((ValueError, RuntimeError)):
            m.load_checkpoint({**w, name: w[name][:-1]})


def test_unknown_kinds_and_sizes_are_refused(groups):
    from neuronx_distributed_amd.models import PokepelConfig, build_model

    def broken(path, value):
        cfg = json.loads(json.dumps(pc.CASES["odd"]))
        node = cfg
        for p in path[:-1]:
            node = node[p]
        node[path[-1]] = value
        return PokepelConfig.from_dict(cfg)

    L = "layers"
    for path, value in (((L, 0, "type"), "other"),
                        ((L, 0, "mlp", "kind"), "other"),
                        ((L, 0, "mlp", "router", "top"), 5),
                        ((L, 0, "mlp", "router", "groups", "count"), 4),
                        ((L, 0, "mixer", "rot", "dims"), 7),
                        ((L, 0, "mixer", "kv_rank"), 1024),
                        ((L, 1, "mixer", "decay"), [0.5]),
                        ((L, 1, "mixer", "dim"), 600),
                        ((L, 1, "mixer", "rot", "dims"), 14)):
        with pytest.raises(ValueError):
            build_model("Pokepel", broken(path, value))


def test_only_the_serving_engine_runs_it(groups):
    from neuronx_distributed_amd.inference import InferenceEngine
    from neuronx_distributed_amd.models import (build_model,
                                                get_pokepel_config)

    m = build_model("Pokepel", get_pokepel_config("pokepel-tiny"))
    with pytest.raises(RuntimeError):
        InferenceEngine(m, 128, 1)
    with pytest.raises(NotImplementedError):
        m(torch.zeros(1, 1, dtype=torch.long))


def test_pools_of_latents_and_memories():
    c = CacheManager([[MatrixState(2, 8, 5)], [PagedLatent(24, 8)]], 200, 2,
                     device="cpu", dtype=torch.bfloat16)
    (S, n, m), latent = c.pools[0][0], c.pools[1][0]
    assert S.shape == (3, 2, 8, 5) and S.dtype == torch.float32
    assert n is None and m is None
    assert latent.shape == (5, 64, 32) and latent.dtype == torch.bfloat16
    assert c.paged and c.window == 0


@pytest.mark.parametrize("base,dims,sc", [
    (1e4, 24, dict(factor=8.0, original=512, fast=16.0, slow=1.0)),
    (5e4, 64, dict(factor=2.0, original=4096, fast=32.0, slow=1.0)),
    # every pair slow; the borders at the first and past the last pair
    (9.0, 6, dict(factor=3.0, original=40, fast=2.5, slow=0.6)),
    (300.0, 16, dict(factor=5.0, original=20, fast=40.0, slow=20.0)),
    (2.0, 8, dict(factor=1.0, original=10000, fast=1.0, slow=0.001)),
    (1e4, 32, dict(factor=40.0, original=2048, fast=9.0, slow=9.0)),
])
def test_scaled_frequencies(base, dims, sc):
    rot = {"base": base, "dims": dims, "scaling": sc}
    got, amp = sv.yarn_frequencies(base, dims, "cpu", sc)
    want = torch.tensor([po.frequency(i, rot) for i in range(dims // 2)],
                        dtype=torch.float64)
    assert got.dtype == torch.float64
    assert torch.allclose(got, want, rtol=1e-14, atol=0)
    assert amp == po.amplitude(rot) == 1.0 + 0.1 * math.log(sc["factor"])


def test_kept_interpolated_and_slowed_pairs():
    rot = {"base": 1e4, "dims": 24, "scaling": dict(
        factor=8.0, original=512, fast=16.0, slow=1.0)}
    r = [po.ramp(i, rot) for i in range(12)]
    assert r[0] == 0.0 and r[-1] == 1.0 and r == sorted(r)
    assert any(0.05 < x < 0.95 for x in r)
    # a pair turns `turns` times in `original` positions at pair_of(turns)
    f = po.frequency(0, {**rot, "scaling": None})
    assert f == 1.0 and 512 * f / (2 * math.pi) > 16.0


# ---------------------------------------------------------------------------
# the oracle's mechanisms against independent forms
# ---------------------------------------------------------------------------

def _r(*s, seed=0):
    return torch.randn(*s, generator=torch.Generator().manual_seed(seed),
                       dtype=torch.float64)


def test_retention_closed_form_and_carried_state():
    T, H, D, E = 13, 2, 5, 3
    q, k, v = _r(T, H, D), _r(T, H, D, seed=1), _r(T, H, E, seed=2)
    decay = [0.8, 1.0]
    o, S = po.retention(q, k, v, decay)
    away = torch.arange(T)[:, None] - torch.arange(T)
    for h in range(H):
        a = torch.where(away >= 0, decay[h] ** away.clamp(min=0).double(),
                        torch.zeros(()).double())
        assert torch.allclose(o[:, h], ((q[:, h] @ k[:, h].T) * a) @ v[:, h])
    o1, S1 = po.retention(q[:6], k[:6], v[:6], decay)
    o2, S2 = po.retention(q[6:], k[6:], v[6:], decay, S1)
    assert torch.allclose(torch.cat([o1, o2]), o) and torch.allclose(S2, S)


def test_a_sink_is_one_more_key_with_a_value_of_zero():
    s, v = _r(9, 9), _r(9, 4, seed=1)
    sink = torch.tensor(0.7).double()
    ahead = torch.ones(9, 9, dtype=torch.bool).triu(1)
    full = torch.cat([s.masked_fill(ahead, -math.inf), sink.expand(9, 1)], 1)
    assert torch.allclose(po.attend(s, v, sink),
                          torch.softmax(full, 1)[:, :9] @ v)


@pytest.mark.parametrize("turn,partner", [(po.rotate_pairs, 1),
                                          (po.rotate_halves, 3)])
def test_rotations(turn, partner):
    rot = {"base": 50.0, "dims": 6}
    q, k = _r(1, 1, 10), _r(1, 1, 10, seed=1)
    dots = [(turn(q, [p + 7], rot) * turn(k, [p], rot)).sum()
            for p in (0, 3, 1000)]
    assert max(dots) - min(dots) < 1e-9
    x = torch.zeros(1, 1, 10).double()
    x[..., 0] = 1.0
    y = turn(x, [math.pi / 2], rot)
    assert abs(y[0, 0, partner] - 1) < 1e-12
    y[..., partner] = 0.0
    assert y.abs().max() < 1e-12
    assert torch.equal(turn(q, [5], rot)[..., 6:], q[..., 6:])
    # the amplitude only scales what turns
    sc = {**rot, "scaling": dict(factor=math.e, original=1e9, fast=2.0,
                                 slow=1.0)}
    y, z = turn(q, [5], rot), turn(q, [5], sc)
    assert torch.allclose(1.1 * y[..., :6], z[..., :6])


def test_poly_norm_of_one_row():
    z = torch.tensor([[1.0, -2.0, 3.0]]).double()
    act = torch.tensor([0.5, 0.25, -0.125, 2.0]).double()
    got = po.poly_norm(z, act, 0.0)[0, 1]
    want = 0.5 * -2 / math.sqrt(14 / 3) + 0.25 * 4 / math.sqrt(98 / 3) \
        - 0.125 * -8 / math.sqrt((1 + 64 + 729) / 3) + 2.0
    assert abs(got - want) < 1e-12


def test_routing_takes_groups_by_their_largest():
    z = torch.tensor([[3.0, -9.0, 2.5, 2.4]]).double()
    idx, w = po.route(z, 2, 1, 2)
    assert idx[0].tolist() == [0, 1]
    assert torch.allclose(w[0], torch.softmax(z[0], 0)[:2])
    assert w.sum() < 0.5


# ---------------------------------------------------------------------------
# the oracle notices planted mistakes (so the GPU comparisons would)
# ---------------------------------------------------------------------------

def _set(path, change):
    def apply(cfg):
        node = cfg
        for p in path[:-1]:
            node = node[p]
        node[path[-1]] = change(node[path[-1]])
    return apply


def _mix(i, *path):
    return ("layers", i, "mixer") + path


MISTAKES = {
    "eps": _set(("norm", "eps"), lambda s: 1e-3),
    "scale": _set(_mix(1, "scale"), lambda s: s * 1.01),
    "amplitude in the scale": _set(_mix(1, "scale"), lambda s: s * 1.1),
    "base of the latent's rotation": _set(_mix(2, "rot", "base"),
                                          lambda s: s * 1.05),
    "base of the retention's": _set(_mix(3, "rot", "base"),
                                    lambda s: s * 1.05),
    "two elements fewer turn": _set(_mix(0, "rot", "dims"), lambda s: s - 2),
    "factor": _set(_mix(2, "rot", "scaling", "factor"), lambda s: s * 1.1),
    "fast": _set(_mix(2, "rot", "scaling", "fast"), lambda s: s * 3),
    "slow": _set(_mix(2, "rot", "scaling", "slow"), lambda s: s * 0.2),
    "original": _set(_mix(2, "rot", "scaling", "original"),
                     lambda s: s * 2),
    "no scaling": _set(_mix(1, "rot", "scaling"), lambda s: None),
    "decays in another order": _set(_mix(3, "decay"), lambda s: s[::-1]),
    "one decay": _set(_mix(0, "decay"), lambda s: s[:1] * 3),
    "one group more": _set(("layers", 2, "mlp", "router", "groups", "keep"),
                           lambda s: s + 1),
    "one expert more": _set(("layers", 0, "mlp", "router", "top"),
                            lambda s: s + 1),
    "no shared expert": _set(("layers", 2, "mlp", "shared"),
                             lambda s: None),
}


def _renormed(z, *a):
    idx, w = ROUTE(z, *a)
    return idx, w / w.sum(1, keepdim=True)


def _softmax_of_the_kept(z, count, keep, top):
    best = z.view(len(z), count, -1).amax(2).topk(keep).indices
    kept = torch.zeros(len(z), count, dtype=torch.bool).scatter_(1, best,
                                                                 True)
    kept = kept.repeat_interleave(z.shape[1] // count, 1)
    return ROUTE(z.masked_fill(~kept, -50.0), count, keep, top)


def _groups_by_sum(z, count, keep, top):
    s = torch.softmax(z, 1)
    score = s.view(len(s), count, -1).topk(2, dim=2).values.sum(2)
    best = score.topk(keep).indices
    kept = torch.zeros(len(s), count, dtype=torch.bool).scatter_(1, best,
                                                                 True)
    m = s.masked_fill(~kept.repeat_interleave(s.shape[1] // count, 1), -1.0)
    idx = m.topk(top).indices
    return idx, s.gather(1, idx)


def _retention(change):
    return lambda q, k, v, a, s=None: RETENTION(*change(q, k, v, a), s)


def _poly_of_normed(z, act, eps):
    n = po.rms(z, eps)
    return act[0] * n + act[1] * n ** 2 + act[2] * n ** 3 + act[3]


ROUTE, RETENTION, ATTEND, PAIRS, HALVES, LATENTS, POLY = (
    po.route, po.retention, po.attend, po.rotate_pairs, po.rotate_halves,
    po.latents, po.poly_norm)
PATCHES = {
    "halves for pairs": {"rotate_pairs": HALVES},
    "pairs for halves": {"rotate_halves": PAIRS},
    "no rotation": {"rotate_halves": lambda x, p, r: x},
    "positions from one": {"rotate_halves": lambda x, p, r: HALVES(
        x, [i + 1 for i in p], {**r, "base": r["base"] * 1.3})},
    "no amplitude": {"amplitude": lambda r: 1.0},
    "no sink": {"attend": lambda s, v, k: ATTEND(
        s, v, torch.full_like(k, -1e30))},
    "scaled sink": {"attend": lambda s, v, k: ATTEND(s, v, 0.3 * k)},
    "latents not normed": {"latents": lambda r, w, n, rot, p, eps: (
        r[:, :n] * w, LATENTS(r, w, n, rot, p, eps)[1])},
    "shared key normed": {"latents": lambda r, w, n, rot, p, eps: LATENTS(
        torch.cat([r[:, :n], po.rms(r[:, n:], eps)], 1), w, n, rot, p, eps)},
    "decays squared": {"retention": _retention(
        lambda q, k, v, a: (q, k, v, [x * x for x in a]))},
    "weights that sum to one": {"route": _renormed},
    "softmax of the kept": {"route": _softmax_of_the_kept},
    "groups by their two largest": {"route": _groups_by_sum},
    "powers of the normed": {"poly_norm": _poly_of_normed},
    "no constant": {"poly_norm": lambda z, a, e: POLY(z, a, e) - a[3]},
    "sigmoid for silu": {"silu": po.sigmoid},
    "no residual gate": {"residual_gate": lambda W, p, h: 1.0},
    "gate without bias": {"residual_gate": lambda W, p, h: po.sigmoid(
        h @ W[p].T)},
    "gates swapped": {"residual_gate": lambda W, p, h: po.sigmoid(
        h @ W[p[:-1] + "1"].T + W[p[:-1] + "1.b"])},
}


@pytest.mark.parametrize("name", list(MISTAKES) + list(PATCHES))
def test_planted_mistakes_show(name, monkeypatch):
    """Every mistake moves some logits by more than five times the float32
    limit of the GPU tests."""
    cfg = json.loads(json.dumps(pc.CASES["mixed"]))
    w = pc.weights(cfg)
    g = torch.Generator().manual_seed(1000)
    toks = torch.randint(0, cfg["vocab"], (110,), generator=g).tolist()
    good = po.forward(cfg, w, toks)
    if name in MISTAKES:
        MISTAKES[name](cfg)
    for fn, new in PATCHES.get(name, {}).items():
        monkeypatch.setattr(po, fn, new)
    bad = po.forward(cfg, w, toks)
    err = (good - bad).pow(2).mean(1).sqrt() / good.pow(2).mean().sqrt()
    assert err.max() > 1e-4, err.max().item()


def test_side_by_side_is_not_one_after_the_other():
    """The feed-forward reads the same rows as the mixer, not its result."""
    cfg, w = pc.CASES["mixed"], pc.weights(pc.CASES["mixed"])
    W = {n: t.double() for n, t in w.items()}
    x = W["embed"][torch.tensor([3, 9, 27])]
    L, eps = cfg["layers"][1], cfg["norm"]["eps"]
    h = po.norm(x, W["l1.norm1"], eps)
    a = po.latent_mixer(W, "l1.mix.", h, L["mixer"], eps) * \
        po.residual_gate(W, "l1.rg1", h)
    side = po.dense_mlp(W, "l1.mlp.", h, L["mlp"], eps)
    after = po.dense_mlp(W, "l1.mlp.", po.norm(x + a, W["l1.norm1"], eps),
                         L["mlp"], eps)
    assert (side - after).abs().max() > 1e-2
