"""What of the Sutuvik design needs no GPU: configuration, weights, state
specifications; and the oracle's own forms and its sensitivity to planted
mistakes."""

import json
import math

import pytest
import torch

import sutuvik_cases as sc
import sutuvik_oracle as so
from neuronx_distributed_amd.inference import (CacheManager, ConvRing,
                                               MatrixState, PagedKV)
from neuronx_distributed_amd.ops import serving as sv


@pytest.fixture
def groups():
    from neuronx_distributed_amd.inference import single_process_groups

    single_process_groups()


# ---------------------------------------------------------------------------
# registry, configuration, weights, state
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("case", list(sc.CASES))
def test_load_pretrained_by_config(case, tmp_path, groups):
    from neuronx_distributed_amd.models import (SutuvikForCausalLM,
                                                load_pretrained)

    cfg = sc.CASES[case]
    w = sc.weights(cfg)
    sc.save(cfg, w, tmp_path)
    m = load_pretrained(str(tmp_path), torch.float32)
    assert isinstance(m, SutuvikForCausalLM)
    assert {p.dtype for p in m.parameters()} == {torch.float32}
    assert torch.equal(m.side_embed, w["side.embed"].float())
    for i, (L, layer) in enumerate(zip(cfg["layers"], m.layers)):
        p, c = f"l{i}.", L["mixer"]
        mix, proj = layer.mix.mixer, layer.mix.proj.weight
        assert torch.equal(layer.conv, w[p + "canon1"].float().t())
        ring = ConvRing(cfg["width"], cfg["canon"]["taps"])
        H = c["heads"]
        if L["type"] == "mamba2":
            full = w[p + "mix.in"].float()
            n = full.shape[0] - H
            assert torch.equal(proj[:n], full[:n])
            assert torch.equal(mix.step_proj, full[n:])
            channels = H * c["vdim"] + 2 * c["groups"] * c["state"]
            assert layer.cache_specs() == [
                ring, MatrixState(H, c["state"], c["vdim"]),
                ConvRing(channels, c["conv"])]
        else:
            names = ["q", "k", "v"] + ["g"] * (L["type"] == "attention")
            full = torch.cat([w[f"{p}mix.{x}"] for x in names]).float()
            n = full.shape[0]
            assert torch.equal(proj[:n], full)
            assert layer.cache_specs() == [
                ring, PagedKV(c["kv_heads"], c["dim"], c["vdim"])]
        assert proj.shape[0] % 8 == 0 and not proj[n:].any()
        f = L["mlp"]
        if f is None:
            assert layer.mlp is None
            continue
        r, ff = f["router"], f["expert"]["ff"]
        assert layer.mlp.routing == sv.Routing(
            r["top"], True, r["groups"]["count"], r["groups"]["keep"])
        assert torch.equal(layer.mlp.bias, w[p + "mlp.correction"].float())
        for e in range(r["experts"]):
            q = f"{p}mlp.e{e}."
            assert torch.equal(layer.mlp.gate_up[e][:ff],
                               w[q + "gate"].float())
            assert torch.equal(layer.mlp.gate_up[e][ff:], w[q + "up"].float())
            assert torch.equal(layer.mlp.down[e], w[q + "down"].float())


def test_bad_checkpoints_are_refused(groups):
    from neuronx_distributed_amd.models import SutuvikConfig, build_model

    cfg = sc.CASES["odd"]
    w = sc.weights(cfg)
    m = build_model("Sutuvik", SutuvikConfig.from_dict(cfg), torch.float32)
    m.load_checkpoint(w)
    for name in ("l1.mix.A_log", "l0.side.norm", "l2.mix.sink"):
        with pytest.raises(KeyError):
            m.load_checkpoint({k: v for k, v in w.items() if k != name})
    with pytest.raises(KeyError):
        m.load_checkpoint({**w, "head": w["embed"]})
    for name in ("embed", "l0.mix.q", "l1.mix.in", "l1.mix.conv",
                 "l0.mlp.correction", "l2.mix.k.norm", "side.embed"):
        with pytest.raises((ValueError, RuntimeError)):
            m.load_checkpoint({**w, name: w[name][:-1]})


def test_unknown_kinds_and_sizes_are_refused(groups):
    from neuronx_distributed_amd.models import SutuvikConfig, build_model

    def broken(path, value):
        cfg = json.loads(json.dumps(sc.CASES["odd"]))
        node = cfg
        for p in path[:-1]:
            node = node[p]
        node[path[-1]] = value
        return SutuvikConfig.from_dict(cfg)

    L = "layers"
    for path, value in (((L, 0, "type"), "other"),
                        ((L, 0, "mlp", "kind"), "other"),
                        ((L, 0, "mlp", "router", "top"), 5),
                        ((L, 0, "mlp", "router", "groups", "count"), 4),
                        ((L, 0, "mixer", "rot", "dims"), 7),
                        ((L, 0, "mixer", "kv_heads"), 2),
                        ((L, 0, "mixer", "dim"), 600),
                        ((L, 1, "mixer", "groups"), 2),
                        ((L, 1, "mixer", "state"), 513),
                        ((L, 1, "mixer", "conv"), 66),
                        ((L, 1, "mixer", "norm_groups"), 2),
                        (("norm", "groups"), 3), (("canon", "taps"), 0)):
        with pytest.raises(ValueError):
            build_model("Sutuvik", broken(path, value))


def test_only_the_serving_engine_runs_it(groups):
    from neuronx_distributed_amd.inference import InferenceEngine
    from neuronx_distributed_amd.models import (build_model,
                                                get_sutuvik_config)

    m = build_model("Sutuvik", get_sutuvik_config("sutuvik-tiny"))
    with pytest.raises(RuntimeError):
        InferenceEngine(m, 128, 1)
    with pytest.raises(NotImplementedError):
        m(torch.zeros(1, 1, dtype=torch.long))


def test_pools_of_rings_and_memories():
    c = CacheManager([[ConvRing(24, 3), MatrixState(2, 8, 5)],
                      [ConvRing(24, 3), PagedKV(1, 8, 16)]], 200, 2,
                     device="cpu", dtype=torch.bfloat16)
    ring, (S, _, _) = c.pools[0]
    assert ring.shape == (3, 3, 24) and ring.dtype == torch.bfloat16
    assert S.shape == (3, 2, 8, 5) and S.dtype == torch.float32
    assert c.paged and c.window == 0 and c.num_pages == 4
    c = CacheManager([[ConvRing(8, 4)]], 64, 1, device="cpu")
    assert not c.paged
    c.admit("a")
    c.extend("a", 60)
    assert c.free_pages == c.num_pages


def test_scaled_frequencies():
    """Kept, interpolated and slowed pairs, all three present."""
    rot = {"base": 1e4, "dims": 24, "scaling": {
        "factor": 8.0, "low": 1.5, "high": 4.0, "original": 512}}
    got = sv.rotary_frequencies(1e4, 24, "cpu", rot["scaling"])
    want = torch.tensor([so.frequency(i, rot) for i in range(12)]).double()
    assert torch.allclose(got, want, rtol=1e-6)
    plain = sv.rotary_frequencies(1e4, 24, "cpu")
    ratio = plain / got
    assert (ratio == 1).any() and (ratio - 8).abs().min() < 1e-9
    assert ((ratio > 1.01) & (ratio < 7.9)).any()


# ---------------------------------------------------------------------------
# the oracle's mechanisms against independent forms
# ---------------------------------------------------------------------------

def _r(*s, seed=0):
    return torch.randn(*s, generator=torch.Generator().manual_seed(seed),
                       dtype=torch.float64)


def test_convolution_and_state_space_closed_forms():
    x, w = _r(20, 3), _r(3, 4, seed=1)
    want = torch.nn.functional.conv1d(
        torch.nn.functional.pad(x.t()[None], (3, 0)), w[:, None], groups=3)
    assert torch.allclose(so.causal_conv(x, w), want[0].t())
    T, H, P, G, N = 12, 4, 3, 2, 5
    x, B, C = _r(T, H, P), _r(T, G, N, seed=1), _r(T, G, N, seed=2)
    dt, skip = _r(T, H, seed=3).abs(), _r(H, seed=4)
    decay = torch.exp(-dt)
    y, S = so.state_space(x, B, C, dt, decay, skip)
    for h in range(H):           # the quadratic form
        g = h // 2
        L = torch.zeros(T, T).double()
        for t in range(T):
            for s in range(t + 1):
                L[t, s] = decay[s + 1:t + 1, h].prod() * dt[s, h]
        want = ((C[:, g] @ B[:, g].T) * L) @ x[:, h] + skip[h] * x[:, h]
        assert torch.allclose(y[:, h], want)
    # in two parts, with the state carried
    y1, S1 = so.state_space(x[:7], B[:7], C[:7], dt[:7], decay[:7], skip)
    y2, S2 = so.state_space(x[7:], B[7:], C[7:], dt[7:], decay[7:], skip, S1)
    assert torch.allclose(torch.cat([y1, y2]), y) and torch.allclose(S2, S)


def test_sinks_and_capped_scores():
    """A sink is one more key with a value of zero."""
    s, v = _r(9, 9), _r(9, 4, seed=1)
    sink = torch.tensor(0.7).double()
    got = so.attend(s, v, sink)
    ahead = torch.ones(9, 9, dtype=torch.bool).triu(1)
    full = torch.cat([s.masked_fill(ahead, -math.inf),
                      sink.expand(9, 1)], 1)
    want = torch.softmax(full, 1)[:, :9] @ v
    assert torch.allclose(got, want)
    z = torch.zeros(()).double()
    e = torch.exp(s.masked_fill(ahead, -math.inf))
    assert torch.allclose(so.attend(s, v, z),
                          (e / (1 + e.sum(1, keepdim=True))) @ v)
    assert so.query_temperature(48, 0.5, 50) == 1.0
    assert so.query_temperature(49, 0.5, 50) == 1.0 + 0.5 * math.log(2.0)
    assert so.slope(7, 8) == 2.0 ** -8


def test_rotation_of_neighbouring_pairs():
    rot = {"base": 50.0, "dims": 6}
    q, k = _r(1, 1, 10), _r(1, 1, 10, seed=1)
    dots = [(so.rotate_pairs(q, [p + 7], rot) *
             so.rotate_pairs(k, [p], rot)).sum() for p in (0, 3, 1000)]
    assert max(dots) - min(dots) < 1e-9
    x = torch.zeros(1, 1, 10).double()
    x[..., 0] = 1.0
    y = so.rotate_pairs(x, [math.pi / 2], rot)
    assert abs(y[0, 0, 1] - 1) < 1e-12 and y[0, 0, 2:].abs().max() == 0
    assert torch.equal(so.rotate_pairs(q, [5], rot)[..., 6:], q[..., 6:])


def test_routing_with_negative_choice_scores():
    z = torch.tensor([[0.0, 3.0, 2.0, 2.5]]).double()
    c = torch.tensor([-0.1, -3.0, -1.5, -1.6]).double()
    # groups: (0.4, -2.05) and (-0.62, -0.68): the second has the larger sum
    idx, w = so.route(z, c, 2, 1, 2)
    assert sorted(idx[0].tolist()) == [2, 3]
    s = so.sigmoid(z)[0]
    assert torch.allclose(w.sum(), torch.ones(()).double())
    assert torch.allclose(w[0, 0] / w[0, 1], s[idx[0, 0]] / s[idx[0, 1]])


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
    "norm in one group": _set(("norm", "groups"), lambda s: 1),
    "eps": _set(("norm", "eps"), lambda s: 1e-3),
    "logit scale": _set(("logit_scale",), lambda s: s * 1.01),
    "output norm in one group": _set(_mix(0, "norm_groups"), lambda s: 1),
    "temperature": _set(_mix(1, "q_temp", "coef"), lambda s: s * 1.02),
    "temperature's step": _set(_mix(1, "q_temp", "every"), lambda s: s + 1),
    "scale": _set(_mix(1, "scale"), lambda s: s * 1.01),
    "base": _set(_mix(2, "rot", "base"), lambda s: s * 1.05),
    "factor": _set(_mix(2, "rot", "scaling", "factor"), lambda s: s * 1.2),
    "high": _set(_mix(2, "rot", "scaling", "high"), lambda s: s * 1.2),
    "low": _set(_mix(2, "rot", "scaling", "low"), lambda s: s * 0.5),
    "cap": _set(_mix(2, "softcap"), lambda s: s * 1.05),
    "no mixing": _set(_mix(2, "v_mix"), lambda s: False),
    "one group more": _set(("layers", 2, "mlp", "router", "groups", "keep"),
                           lambda s: s + 1),
    "one expert more": _set(("layers", 0, "mlp", "router", "top"),
                            lambda s: s + 1),
}


def _half_pairs(x, positions, rot):
    n = rot["dims"]
    order = [i // 2 + (n // 2) * (i % 2) for i in range(n)]
    out = x.clone()
    out[..., order] = ROTATE(x[..., order], positions, rot)[..., :n]
    return out


def _anti_causal(x, w):
    return CONV(x, w.flip(1))


def _route_weights_with_correction(z, c, groups, keep, top):
    idx, _ = ROUTE(z, c, groups, keep, top)
    w = (so.sigmoid(z) + c).gather(1, idx)
    return idx, w / w.sum(1, keepdim=True)


def _route_groups_by_largest(z, c, groups, keep, top):
    s = so.sigmoid(z) + c
    best = s.view(len(s), groups, -1).amax(2).topk(keep).indices
    keep = torch.zeros(len(s), groups, dtype=torch.bool).scatter_(1, best,
                                                                 True)
    s = s.masked_fill(~keep.repeat_interleave(s.shape[1] // groups, 1),
                      -math.inf)
    idx = s.topk(top).indices
    w = so.sigmoid(z).gather(1, idx)
    return idx, w / w.sum(1, keepdim=True)


def _mixed_backwards(v, lam, first):
    return v if first is None else MIXED(first, lam, v)


ROTATE, CONV, ROUTE, MIXED = (so.rotate_pairs, so.causal_conv, so.route,
                              so.mixed_values)
SPACE, ATTEND = so.state_space, so.attend
PATCHES = {
    "half pairs": {"rotate_pairs": _half_pairs},
    "no rotation": {"rotate_pairs": lambda x, p, r: x},
    "filter the other way": {"causal_conv": _anti_causal},
    "no sink": {"attend": lambda s, v, k: ATTEND(
        s, v, torch.full_like(k, -1e30))},
    "no bias": {"slope": lambda h, H: 0.0},
    "slopes from zero": {"slope": lambda h, H: 2.0 ** (-8.0 * h / H)},
    "no skip": {"state_space": lambda x, B, C, dt, a, d, s=None: SPACE(
        x, B, C, dt, a, 0 * d, s)},
    "input without step": {
        "state_space": lambda x, B, C, dt, a, d, s=None: SPACE(
            x, B, C, torch.ones_like(dt), a, d, s)},
    "heads share keys in turn": {
        "state_space": lambda x, B, C, dt, a, d, s=None: SPACE(
            x, B.flip(1), C.flip(1), dt, a, d, s)},
    "weights with correction": {"route": _route_weights_with_correction},
    "groups by their largest": {"route": _route_groups_by_largest},
    "shares swapped": {"mixed_values": _mixed_backwards},
    "plain gelu": {"gelu_tanh": lambda z: z * so.sigmoid(1.702 * z)},
    "temperature of the next": {"query_temperature": lambda p, c, e: 1.0
                                + c * math.log((p + 2) // e + 1)},
    "no token input": {"token_side": lambda W, p, x, e, eps: 0 * x},
}


@pytest.mark.parametrize("name", list(MISTAKES) + list(PATCHES))
def test_planted_mistakes_show(name, monkeypatch):
    """Every mistake moves some logits by more than five times the float32
    limit of the GPU tests."""
    cfg = json.loads(json.dumps(sc.CASES["mixed"]))
    w = sc.weights(cfg)
    g = torch.Generator().manual_seed(1000)
    toks = torch.randint(0, cfg["vocab"], (110,), generator=g).tolist()
    good = so.forward(cfg, w, toks)
    if name in MISTAKES:
        MISTAKES[name](cfg)
    for fn, new in PATCHES.get(name, {}).items():
        monkeypatch.setattr(so, fn, new)
    bad = so.forward(cfg, w, toks)
    err = (good - bad).pow(2).mean(1).sqrt() / good.pow(2).mean().sqrt()
    assert err.max() > 1e-4, err.max().item()
