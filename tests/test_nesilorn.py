"""What of the Nesilorn design needs no GPU: configuration, weights, cache
accounting, the tables of a step; and the oracle's own sensitivity to planted
mistakes."""

import json
import math

import numpy as np
import pytest
import torch

import nesilorn_cases as nc
import nesilorn_oracle as no
from neuronx_distributed_amd.inference import (CacheManager, PagedKV,
                                               PagedLatent)
from neuronx_distributed_amd.ops import serving as sv


@pytest.fixture
def groups():
    from neuronx_distributed_amd.inference import single_process_groups

    single_process_groups()


# ---------------------------------------------------------------------------
# registry, configuration, weights
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("case", list(nc.CASES))
def test_load_pretrained_by_config(case, tmp_path, groups):
    from neuronx_distributed_amd.models import (NesilornForCausalLM,
                                                load_pretrained)

    cfg = nc.CASES[case]
    w = nc.weights(cfg)
    nc.save(cfg, w, tmp_path)
    m = load_pretrained(str(tmp_path), torch.float32)
    assert isinstance(m, NesilornForCausalLM)
    assert {p.dtype for p in m.parameters()} == {torch.float32}
    assert torch.equal(m.embed.weight, w["embed"].float())
    for i, (L, layer) in enumerate(zip(cfg["layers"], m.layers)):
        p, c = f"l{i}.", L["mixer"]
        mix = layer.mix.mixer
        assert mix.cache_specs() == [PagedLatent(
            c["kv_rank"], c["rot_dim"], (c["mask"] or {}).get("size", 0))]
        assert torch.equal(layer.mix.proj.weight, torch.cat(
            [w[f"{p}mix.{n}"] for n in ("q", "dkv", "g")]).float())
        H, D, R = c["heads"], c["dim"], c["kv_rank"]
        uk = w[p + "mix.uk"].float()
        for h in range(H):       # both forms of W_uk
            assert torch.equal(mix.absorb[h].T, uk[h * D:(h + 1) * D])
        assert torch.equal(mix.expand, torch.cat(
            [uk, w[p + "mix.uv"].float()]))
        f = L["mlp"]
        if f is None:
            assert layer.mlp is None
        elif f["kind"] == "moe":
            ff = f["expert"]["ff"]
            for e in range(f["router"]["experts"]):
                q = f"{p}mlp.e{e}."
                assert torch.equal(layer.mlp.gate_up[e][:ff],
                                   w[q + "gate"].float())
                assert torch.equal(layer.mlp.gate_up[e][ff:],
                                   w[q + "up"].float())
                assert torch.equal(layer.mlp.down[e], w[q + "down"].float())
            assert layer.mlp.act[1] == f["expert"]["limit"]


def test_bad_checkpoints_are_refused(groups):
    from neuronx_distributed_amd.models import NesilornConfig, build_model

    cfg = nc.CASES["odd"]
    w = nc.weights(cfg)
    m = build_model("Nesilorn", NesilornConfig.from_dict(cfg), torch.float32)
    with pytest.raises(KeyError):
        m.load_checkpoint({k: v for k, v in w.items()
                           if k != "l1.mlp.e2.down"})
    with pytest.raises(KeyError):
        m.load_checkpoint({**w, "head": w["embed"]})
    for name in ("embed", "l0.mix.q", "l0.mix.uk", "l1.mlp.router.b",
                 "l0.mlp.e1.gate"):
        with pytest.raises((ValueError, RuntimeError)):
            m.load_checkpoint({**w, name: w[name][:-1]})


def test_unknown_kinds_and_sizes_are_refused(groups):
    from neuronx_distributed_amd.models import NesilornConfig, build_model

    def broken(path, value):
        cfg = json.loads(json.dumps(nc.CASES["odd"]))
        node = cfg["layers"][0]
        for p in path[:-1]:
            node = node[p]
        node[path[-1]] = value
        return NesilornConfig.from_dict(cfg)

    for path, value in ((("type",), "other"), (("mlp", "kind"), "other"),
                        (("mlp", "router", "top"), 4),
                        (("mlp", "router", "experts"), 600),
                        (("mixer", "rot", "dims"), 8),
                        (("mixer", "rot", "dims"), 5),
                        (("mixer", "kv_rank"), 1020)):
        with pytest.raises(ValueError):
            build_model("Nesilorn", broken(path, value))


def test_only_the_serving_engine_runs_it(groups):
    from neuronx_distributed_amd.inference import InferenceEngine
    from neuronx_distributed_amd.models import NesilornConfig, build_model

    m = build_model("Nesilorn", NesilornConfig.from_dict(nc.CASES["odd"]))
    with pytest.raises(RuntimeError):
        InferenceEngine(m, 128, 1)
    with pytest.raises(NotImplementedError):
        m(torch.zeros(1, 1, dtype=torch.long))


# ---------------------------------------------------------------------------
# cache and step tables
# ---------------------------------------------------------------------------

@pytest.mark.parametrize("window", [1, 64, 65, 130, 200])
@pytest.mark.parametrize("step", [1, 2, 37, 64, 100])
def test_pages_and_spans_hold_every_visible_key(window, step):
    """Pages behind the window return; the gathered span of a portion has a
    place, with the right page in it, for every key that a row sees."""
    c = CacheManager([[PagedLatent(8, 4, window)]], 64 * 30, 1)
    c.admit("a")
    length = 0
    while length + step <= 1300:
        st = c.extend("a", step)
        row = np.zeros(c.table_width, dtype=np.int32)
        c.table_row(st, row)
        pages, table = sv.key_spans([(st.slot, 0, step, length)], [row],
                                    window)
        seen = [j for i in {length, length + step // 2, length + step - 1}
                for j in range(i + 1) if no.visible(i, j, window)]
        for j in seen:
            assert st.pages[j // 64] >= 0
            assert pages[table[0][j // 64]] == st.pages[j // 64]
        assert len(pages) <= -(-(window + step) // 64) + 1
        assert max(table[0]) < len(pages)
        st.length += step
        length += step
        live = [p for p in st.pages if p >= 0]
        assert len(set(live)) == len(live)
        assert len(live) + c.free_pages == c.num_pages


def test_spans_of_several_portions_follow_each_other():
    rows = np.arange(24, dtype=np.int32).reshape(2, 12)
    pages, table = sv.key_spans([(0, 0, 70, 130), (1, 70, 3, 0)], rows, 0)
    assert pages == [0, 1, 2, 3, 12]
    assert table[0][:4] == [0, 1, 2, 3] and table[1][0] == 4
    pages, table = sv.key_spans([(0, 0, 70, 130), (1, 70, 3, 300)], rows, 64)
    assert pages == [1, 2, 3, 15, 16]    # keys from 67 and from 237 on
    assert table[0][1:4] == [0, 1, 2] and table[1][3:5] == [3, 4]


def test_pools_and_mixed_specs():
    c = CacheManager([[PagedLatent(24, 8, 70)], [PagedKV(2, 8, 16, 100, 3)]],
                     200, 2, device="cpu", dtype=torch.bfloat16)
    assert c.pools[0][0].shape == (5, 64, 32)
    assert c.pools[0][0].dtype == torch.bfloat16
    assert c.window == 100 and c.keep_first == 3 and c.paged


# ---------------------------------------------------------------------------
# the oracle's mechanisms against independent forms
# ---------------------------------------------------------------------------

def test_rotation_depends_on_distance_only():
    g = torch.Generator().manual_seed(0)
    q, k = torch.randn(2, 1, 10, generator=g, dtype=torch.float64)
    dots = [(no.rotate(q, [p + 7], 50.0) * no.rotate(k, [p], 50.0)).sum()
            for p in (0, 3, 1000)]
    assert max(dots) - min(dots) < 1e-9
    assert torch.equal(no.rotate(q, [0], 50.0), q)
    # the pair (i, i + n/2) turns together: a quarter turn of pair 0
    x = torch.zeros(1, 4, dtype=torch.float64)
    x[0, 0] = 1.0
    y = no.rotate(x, [math.pi / 2], 9.0)
    assert torch.allclose(y, torch.tensor([[0, 0, 1.0, 0]]).double())


def test_router_and_activation_closed_forms():
    z = torch.tensor([[0.0, 2.0, -1.0, 2.0 + math.log(3.0)]]).double()
    idx, w = no.route(z, 2)
    assert idx.tolist() == [[3, 1]]
    assert torch.allclose(w, torch.tensor([[0.75, 0.25]]).double())
    got = no.clamped_glu(torch.tensor([5.0, -9.0, 0.5]),
                         torch.tensor([-7.0, 7.0, 0.25]), 2.0)
    s = lambda x: x / (1 + math.exp(-1.702 * x))
    want = [s(2.0) * -1.0, s(-9.0) * 3.0, s(0.5) * 1.25]
    assert torch.allclose(got, torch.tensor(want))
    assert torch.allclose(no.gelu_tanh(torch.linspace(-4, 4, 9)),
                          torch.nn.functional.gelu(torch.linspace(-4, 4, 9),
                                                   approximate="tanh"))


def test_absorbed_form_equals_expanded_form():
    """q . (W_uk c) is (W_uk^T q) . c, and a weighted sum of values is W_uv of
    the weighted sum of latents."""
    g = torch.Generator().manual_seed(1)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    cfg = nc.mixer(3, 6, 4, 5, 9, 4, 0.6)
    T, H, D, P, E, R = 11, 3, 6, 4, 5, 9
    q, c, kr = r(T, H * (D + P)), r(T, R), r(T, P)
    uk, uv = r(H * D, R), r(H * E, R)
    want = no.latent_attention(q, c, kr, uk, uv, cfg, range(T))
    qh = q.view(T, H, D + P)
    ql = torch.stack([torch.cat([
        qh[:, h, :D] @ uk[h * D:(h + 1) * D],
        no.rotate(qh[:, h, D:], range(T), 1e4)], 1) for h in range(H)], 1)
    keys = torch.cat([c, kr], 1)[:, None].expand(T, H, R + P)
    lat = no.window_attention(ql, keys, c[:, None].expand(T, H, R), 0.6, 4)
    got = torch.cat([lat[:, h] @ uv[h * E:(h + 1) * E].T for h in range(H)],
                    1)
    assert torch.allclose(got, want)


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


MIX = ("layers", 0, "mixer")
MISTAKES = {
    "window one short": _set(MIX + ("mask", "size"), lambda s: s - 1),
    "window one long": _set(MIX + ("mask", "size"), lambda s: s + 1),
    "scale": _set(MIX + ("scale",), lambda s: s * 1.01),
    "base": _set(MIX + ("rot", "base"), lambda s: s * 1.05),
    "embedding scale": _set(("embedding", "scale"), lambda s: s * 1.01),
    "limit": _set(("layers", 0, "mlp", "expert", "limit"),
                  lambda s: s * 1.02),
    "one expert more": _set(("layers", 0, "mlp", "router", "top"),
                            lambda s: s + 1),
    "eps": _set(("norm", "eps"), lambda s: 1e-3),
}
PATCHES = {
    "norms around one": {"centred_norm": lambda x, w, eps: no.rms(x, eps) * w},
    "latents not normed": {"plain_norm": lambda x, w, eps: x * w},
    "equal weights": {"route": lambda z, top: (
        z.topk(top).indices, torch.full_like(z[:, :top], 1 / top))},
    "no rotation": {"rotate": lambda x, p, b: x},
    "interleaved pairs": {"rotate": lambda x, p, b: _interleaved(x, p, b)},
    "plain gelu": {"gelu_tanh": lambda z: z * no.sigmoid(1.702 * z)},
    "no shift": {"clamped_glu": lambda g, u, m: GLU(g, u, m) - GLU(
        g, torch.zeros_like(u), m)},
    "one-sided clamp": {"clamped_glu": lambda g, u, m: torch.minimum(
        g, torch.full_like(g, m)) * no.sigmoid(1.702 * torch.minimum(
            g, torch.full_like(g, m))) * (torch.minimum(
                u, torch.full_like(u, m)) + 1.0)},
    "no output gate": {"sigmoid": lambda x: torch.ones_like(x)},
}


def _interleaved(x, positions, base):
    n = x.shape[-1]
    order = [*range(0, n, 2), *range(1, n, 2)]
    return ROTATE(x[..., order], positions, base)[
        ..., np.argsort(order).tolist()]


ROTATE, GLU = no.rotate, no.clamped_glu


@pytest.mark.parametrize("name", list(MISTAKES) + list(PATCHES))
def test_planted_mistakes_show(name, monkeypatch):
    """Every mistake moves some logits by more than five times the float32
    limit of the GPU tests."""
    cfg = json.loads(json.dumps(nc.CASES["mixed"]))
    w = nc.weights(cfg)
    g = torch.Generator().manual_seed(1000)
    toks = torch.randint(0, cfg["vocab"], (110,), generator=g).tolist()
    good = no.forward(cfg, w, toks)
    if name in MISTAKES:
        MISTAKES[name](cfg)
    for fn, new in PATCHES.get(name, {}).items():
        monkeypatch.setattr(no, fn, new)
    bad = no.forward(cfg, w, toks)
    err = (good - bad).pow(2).mean(1).sqrt() / good.pow(2).mean().sqrt()
    assert err.max() > 1e-4, err.max().item()
