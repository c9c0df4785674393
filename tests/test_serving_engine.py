"""Page and slot accounting, the scheduler, the registry and the Voletar
configuration — everything of the serving engine that needs no GPU — and
the oracle's own sensitivity to planted mistakes."""

import json

import numpy as np
import pytest
import torch

import voletar_cases as vc
import voletar_oracle as vo
from neuronx_distributed_amd.inference import (CacheFull, CacheManager,
                                               MatrixState, PagedKV,
                                               Scheduler)


# ---------------------------------------------------------------------------
# cache manager
# ---------------------------------------------------------------------------

def _manager(specs, max_tokens=640, max_seqs=3, max_context=None):
    return CacheManager(specs, max_tokens, max_seqs, max_context)


def _grow(c, rid, n):
    st = c.extend(rid, n)
    st.length += n
    return st


@pytest.mark.parametrize("window,keep", [(1, 0), (64, 0), (65, 1), (92, 22),
                                         (130, 130), (63, 64), (200, 65)])
@pytest.mark.parametrize("step", [1, 2, 37, 64, 100])
def test_pages_behind_the_window_return_and_no_needed_page_does(window, keep,
                                                                step):
    c = _manager([[PagedKV(1, 8, 8, window, keep)]], 64 * 40, 1)
    c.admit("a")
    mask = {"size": window, "keep_first": keep}
    length = 0
    while length + step <= 64 * 40 and length < 1200:
        st = c.extend("a", step)
        # every key a new token sees has a page of its own
        for i in {length, length + step - 1, length + step // 2}:
            for j in range(i + 1):
                if vo.visible(i, j, mask):
                    assert st.pages[j // 64] >= 0, (i, j)
        st.length += step
        length += step
        live = [p for p in st.pages if p >= 0]
        assert len(set(live)) == len(live)
        assert len(live) + c.free_pages == c.num_pages
        bound = -(-keep // 64) + -(-(window + step) // 64) + 2
        assert len(live) <= bound, (length, len(live))
    c.free("a")
    assert c.free_pages == c.num_pages and c.free_slots == 1


def test_release_follows_the_widest_window():
    wide = [[PagedKV(1, 8, 8, 64, 0)], [PagedKV(1, 8, 8, 300, 70)]]
    c = _manager(wide, 64 * 20, 1)
    c.admit("a")
    st = _grow(c, "a", 640)
    c.extend("a", 1)
    # first visible key: 640 - 300 + 1 = 341 -> pages 0..4 are behind, and
    # pages 0 and 1 hold kept tokens
    assert [p >= 0 for p in st.pages] == [True, True] + [False] * 3 + \
        [True] * 6
    full = _manager([[PagedKV(1, 8, 8, 64, 0)], [PagedKV(1, 8, 8)]],
                    64 * 20, 1)
    full.admit("a")
    st = _grow(full, "a", 640)
    full.extend("a", 1)
    assert all(p >= 0 for p in st.pages)   # a causal layer needs them all


def test_all_or_nothing_and_reuse():
    c = _manager([[PagedKV(1, 8, 8), MatrixState(1, 8, 8)]], 256, 2)
    a = c.admit("a")
    _grow(c, "a", 130)
    b = c.admit("b")
    assert a.slot != b.slot
    with pytest.raises(CacheFull):
        c.admit("c")
    with pytest.raises(ValueError):
        c.admit("a")
    with pytest.raises(CacheFull):
        c.extend("b", 65)
    assert c.free_pages == 1 and not b.pages
    _grow(c, "b", 64)
    pages = list(a.pages)
    c.free("a")
    d = c.admit("d")
    assert d.slot == a.slot and d.length == 0
    _grow(c, "d", 190)
    assert sorted(d.pages) == sorted(pages)
    row = np.zeros(c.table_width, dtype=np.int32)
    c.table_row(d, row)
    assert row[:3].tolist() == d.pages and (row[3:] == c.spare_page).all()


def test_context_limit_and_memory_only_models():
    c = _manager([[MatrixState(2, 8, 8, True)]], 64, 1, max_context=5000)
    c.admit("a")
    _grow(c, "a", 4999)            # no pages are needed
    assert c.free_pages == 1 and c.table_width == 1
    _grow(c, "a", 1)
    with pytest.raises(CacheFull):
        c.extend("a", 1)


def test_pool_shapes():
    c = CacheManager([[PagedKV(2, 8, 24, 10, 1), MatrixState(3, 4, 33, True)],
                      [MatrixState(1, 2, 3)]], 100, 4, device="cpu")
    (kc, vc_), (S, n, m) = c.pools[0]
    assert kc.shape == (3, 2, 64, 8) and vc_.shape == (3, 2, 64, 24)
    assert S.shape == (5, 3, 4, 33) and S.dtype == torch.float32
    assert n.shape == (5, 3, 2, 4) and m.shape == (5, 3, 2)
    assert c.pools[1][0][1] is None


# ---------------------------------------------------------------------------
# scheduler (an engine that counts tokens instead of computing)
# ---------------------------------------------------------------------------

class CountingEngine:
    """Next token = (sum of the request's tokens) mod 50."""

    def __init__(self, max_tokens, max_seqs, window=0):
        self.cache = _manager([[PagedKV(1, 8, 8, window)]], max_tokens,
                              max_seqs)
        self.sums, self.steps = {}, []

    def finish(self, rid):
        self.cache.free(rid)

    def step(self, entries):
        assert len({e.id for e in entries}) == len(entries)
        rows = []
        for e in entries:
            if e.id not in self.cache.requests:
                self.cache.admit(e.id)
            _grow(self.cache, e.id, len(e.tokens))
            for p, t in enumerate(e.tokens):
                self.sums[e.id] = self.sums.get(e.id, 0) + t
                if p in e.want:
                    row = torch.zeros(50)
                    row[self.sums[e.id] % 50] = 1.0
                    rows.append(row)
        self.steps.append([(e.id, len(e.tokens)) for e in entries])
        return torch.stack(rows) if rows else None


def _counted(prompt, n):
    s, out = sum(prompt), []
    for _ in range(n):
        out.append(s % 50)
        s += out[-1]
    return out


@pytest.mark.parametrize("budget", [1, 5, 64, 4096])
@pytest.mark.parametrize("slots,tokens", [(1, 256), (3, 512), (8, 4096)])
def test_scheduler_runs_everything(budget, slots, tokens):
    from neuronx_distributed_amd.inference import single_process_groups

    single_process_groups()
    eng = CountingEngine(tokens, slots)
    s = Scheduler(eng, max_step_tokens=budget)
    prompts = [[(7 * i + j) % 50 for j in range(n)]
               for i, n in enumerate((3, 150, 1, 64, 20, 199, 2))]
    reqs = [s.submit(p, 1 + i) for i, p in enumerate(prompts)]
    done = s.run()
    assert sorted(r.id for r in done) == [r.id for r in reqs]
    for i, (r, p) in enumerate(zip(reqs, prompts)):
        assert r.output == _counted(p, 1 + i)
    for step in eng.steps:
        assert sum(n for _, n in step) <= budget
        assert len(step) <= slots
    if slots > 1 and budget > 60:   # portions run beside decoded tokens
        assert any(min(n for _, n in st) == 1 < max(n for _, n in st)
                   for st in eng.steps)
    assert eng.cache.free_pages == eng.cache.num_pages
    assert eng.cache.free_slots == slots


def test_scheduler_stops_at_eos_and_refuses_what_cannot_fit():
    from neuronx_distributed_amd.inference import single_process_groups

    single_process_groups()
    eng = CountingEngine(256, 2)
    s = Scheduler(eng)
    want = _counted([3, 4], 9)
    r = s.submit([3, 4], 9, eos_token_id=want[2])
    with pytest.raises(ValueError):
        s.submit([1] * 250, 7)
    with pytest.raises(ValueError):
        s.submit([], 3)
    assert s.submit([1], 0).output == []
    s.run()
    assert r.output == want[:3]


# ---------------------------------------------------------------------------
# registry, configuration, weights
# ---------------------------------------------------------------------------

@pytest.fixture
def groups():
    from neuronx_distributed_amd.inference import single_process_groups

    single_process_groups()


@pytest.mark.parametrize("case", list(vc.CASES))
def test_load_pretrained_by_config(case, tmp_path, groups):
    from neuronx_distributed_amd.models import (VoletarForCausalLM,
                                                load_pretrained)

    cfg = vc.CASES[case]
    w = vc.weights(cfg)
    vc.save(cfg, w, tmp_path)
    m = load_pretrained(str(tmp_path), torch.float32)
    assert isinstance(m, VoletarForCausalLM)
    assert next(m.parameters()).dtype == torch.float32
    assert m.runs == vo.schedule(cfg)
    assert len(m.cache_specs()) == len(vo.schedule(cfg))
    assert torch.equal(m.head.weight, w["head"].float())
    for i, L in enumerate(cfg["layers"]):
        mix = m.layers[i].mix
        parts = ["q", "k", "v", "g"] if L["type"] == "lightning" else \
            ["left.q", "left.k", "left.v", "right.q", "right.k", "right.v",
             "right.g"]
        assert torch.equal(mix.proj.weight, torch.cat(
            [w[f"l{i}.mix.{n}"] for n in parts]).float())


def test_bad_checkpoints_are_refused(groups):
    from neuronx_distributed_amd.models import VoletarConfig, build_model

    cfg = vc.CASES["odd"]
    w = vc.weights(cfg)
    m = build_model("Voletar", VoletarConfig.from_dict(cfg), torch.float32)
    missing = {k: v for k, v in w.items() if k != "l1.mix.right.f.b"}
    with pytest.raises(KeyError):
        m.load_checkpoint(missing)
    with pytest.raises(KeyError):
        m.load_checkpoint({**w, "l9.extra": w["head"]})
    with pytest.raises(ValueError):
        m.load_checkpoint({**w, "head": w["head"][:, :-1]})
    with pytest.raises(ValueError):
        m.load_checkpoint({**w, "l0.mix.q": w["l0.mix.q"][:-1]})


def test_unknown_kinds_are_refused(tmp_path, groups):
    from neuronx_distributed_amd.models import (VoletarConfig, build_model,
                                                load_pretrained)

    for change in ({"type": "other"}, {"mlp": {"kind": "other", "ff": 8}}):
        cfg = json.loads(json.dumps(vc.CASES["odd"]))
        cfg["layers"][0].update(change)
        with pytest.raises(ValueError):
            build_model("Voletar", VoletarConfig.from_dict(cfg))
    (tmp_path / "config.json").write_text(json.dumps(
        {"architecture": "Nobody"}))
    with pytest.raises(ValueError, match="Nobody"):
        load_pretrained(str(tmp_path))
    with pytest.raises(ValueError):
        VoletarConfig.from_dict({**vc.CASES["odd"], "loop": {
            "start": 1, "stop": 9, "times": 2}}).schedule()


def test_registry_loads_llama(tmp_path, groups):
    """The registry is the framework's: a llama folder loads and generates
    like the model built by hand."""
    from safetensors.torch import save_file

    from neuronx_distributed_amd.inference import generate
    from neuronx_distributed_amd.models import (LlamaForCausalLM, get_config,
                                                load_pretrained)
    from neuronx_distributed_amd.overrides import \
        convert_to_hf_llama_state_dict

    c = get_config("tiny")
    torch.manual_seed(0)
    ref = LlamaForCausalLM(c).eval()
    save_file({k: v.contiguous() for k, v in
               convert_to_hf_llama_state_dict(ref.state_dict()).items()},
              str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps({
        "architectures": ["LlamaForCausalLM"],
        "hidden_size": c.hidden_size, "vocab_size": c.vocab_size,
        "intermediate_size": c.intermediate_size,
        "num_hidden_layers": c.num_hidden_layers,
        "num_attention_heads": c.num_attention_heads,
        "num_key_value_heads": c.num_key_value_heads,
        "max_position_embeddings": c.max_position_embeddings,
        "rms_norm_eps": c.rms_norm_eps, "rope_theta": c.rope_theta}))
    m = load_pretrained(str(tmp_path), torch.float32)
    x = torch.randint(0, c.vocab_size, (2, 7))
    assert torch.equal(generate(m, x, 5), generate(ref, x, 5))


def test_engine_refuses_the_cpu_and_unfit_models(groups):
    from neuronx_distributed_amd.inference import InferenceEngine
    from neuronx_distributed_amd.models import VoletarConfig, build_model

    m = build_model("Voletar", VoletarConfig.from_dict(vc.CASES["odd"]))
    with pytest.raises(RuntimeError):
        InferenceEngine(m, 128, 1)
    with pytest.raises(TypeError):
        InferenceEngine(torch.nn.Linear(2, 2), 128, 1)
    with pytest.raises(NotImplementedError):
        m(torch.zeros(1, 1, dtype=torch.long))


# ---------------------------------------------------------------------------
# the oracle notices planted mistakes (so the GPU comparisons would)
# ---------------------------------------------------------------------------

def _logits(case, tokens, change=None, patch=None, monkeypatch=None):
    cfg = json.loads(json.dumps(vc.CASES[case]))
    if change:
        change(cfg)
    if patch:
        with monkeypatch.context() as mp:
            for name, fn in patch.items():
                mp.setattr(vo, name, fn)
            return vo.forward(cfg, vc.weights(vc.CASES[case]), tokens)
    return vo.forward(cfg, vc.weights(vc.CASES[case]), tokens)


def _set(path, value):
    def change(cfg):
        node = cfg
        for p in path[:-1]:
            node = node[p]
        node[path[-1]] = value(node[path[-1]]) if callable(value) else value
    return change


LEFT = ("layers", 0, "mixer", "left")
MISTAKES = {
    "window one short": _set(LEFT + ("mask", "size"), lambda s: s - 1),
    "window one long": _set(LEFT + ("mask", "size"), lambda s: s + 1),
    "one kept token less": _set(LEFT + ("mask", "keep_first"),
                                lambda s: s - 1),
    "one kept token more": _set(LEFT + ("mask", "keep_first"),
                                lambda s: s + 1),
    "scale": _set(LEFT + ("scale",), lambda s: s * 1.01),
    "cap of the gates": _set(("layers", 0, "mixer", "right", "gate_cap"),
                             lambda s: s * 1.05),
    "a decay": _set(("layers", 1, "mixer", "decay", 2), 0.999),
    "loop of another layer": _set(("loop", "stop"), 3),
    "eps": _set(("norm", "eps"), 1e-3),
    "logit cap": _set(("logit_softcap",), 24.0),
}
PATCHES = {
    "no normaliser floor": {"gated_memory": lambda q, k, v, i, f:
                            _no_floor(q, k, v, i, f)},
    "plain relu": {"relu_squared": lambda x: torch.clamp(x, min=0)},
    "silu left out": {"silu": lambda x: x},
}


def _no_floor(q, k, v, i, f):
    """The gated memory whose normaliser is |n . q| alone.  (Where the
    running maximum starts does not show: m only rescales S and n.)"""
    T, H, D = q.shape
    S, n = q.new_zeros(H, D, v.shape[2]), q.new_zeros(H, D)
    m, out = q.new_zeros(H), []
    for t in range(T):
        mn = torch.maximum(f[t] + m, i[t])
        a, b = torch.exp(f[t] + m - mn), torch.exp(i[t] - mn)
        S = a[:, None, None] * S + b[:, None, None] * (
            k[t][:, :, None] * v[t][:, None, :])
        n, m = a[:, None] * n + b[:, None] * k[t], mn
        den = (n * q[t]).sum(1).abs()
        out.append((S * q[t][:, :, None]).sum(1) / (den[:, None] + 1e-6))
    return torch.stack(out), None


@pytest.mark.parametrize("name", list(MISTAKES) + list(PATCHES))
def test_planted_mistakes_show(name, monkeypatch):
    """Every mistake moves some logits by more than five times the float32
    limit of the GPU tests."""
    g = torch.Generator().manual_seed(1000)
    toks = torch.randint(0, 210, (120,), generator=g).tolist()
    good = _logits("middle_loop", toks)
    bad = _logits("middle_loop", toks, MISTAKES.get(name), PATCHES.get(name),
                  monkeypatch)
    err = (good - bad).pow(2).mean(1).sqrt() / good.pow(2).mean().sqrt()
    assert err.max() > 1e-4, err.max().item()


def test_oracle_recurrences_agree_with_unrolled_sums():
    """The two memories against their closed forms."""
    T, H, D, E = 12, 2, 3, 4
    g = torch.Generator().manual_seed(0)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    q, k, v = r(T, H, D), r(T, H, D), r(T, H, E)
    decay = torch.tensor([0.9, 0.3]).double()
    o, _ = vo.decayed_memory(q, k, v, decay)
    i, f = 4 * r(T, H), vo.log_sigmoid(3 * r(T, H))
    og, _ = vo.gated_memory(q, k, v, i, f)
    for t in range(T):
        for h in range(H):
            a = sum(decay[h] ** (t - s) * (q[t, h] @ k[s, h]) * v[s, h]
                    for s in range(t + 1))
            assert torch.allclose(o[t, h], a)
            # unstabilised: weights e^(F_t - F_s + i_s), floor 1
            w = [torch.exp(f[s + 1:t + 1, h].sum() + i[s, h])
                 for s in range(t + 1)]
            num = sum(x * (q[t, h] @ k[s, h]) * v[s, h]
                      for s, x in enumerate(w))
            den = sum(x * (q[t, h] @ k[s, h]) for s, x in enumerate(w))
            m = max([f[:t + 1, h].sum()] + [x.log() for x in w])
            want = num / (max(den.abs(), torch.ones(())) + 1e-6 * m.exp())
            assert torch.allclose(og[t, h], want, rtol=1e-9)
