"""Pokepel on the serving engine against the plain implementation: whole
prompts, portions, decoding, mixed batches, reused pages and slots."""

import json
import os
import subprocess
import sys

import pytest
import torch

import pokepel_cases as pc
import pokepel_oracle as po

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# rms error over the vocabulary, divided by the rms of the logits.  In bf16 the
# limit of a position is at least four times what rounding the norms and
# activations alone does there; a close call of a router, decided the other way,
# moves a position all the same: one in fifty, and at least one, may be over.
LIMIT = {torch.float32: 2e-5, torch.bfloat16: 5e-2}
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module", autouse=True)
def _groups():
    from neuronx_distributed_amd.inference import single_process_groups
    from neuronx_distributed_amd.ops import serving

    serving.ensure_built()
    single_process_groups()


_models, _want = {}, {}


def _model(case, dtype):
    from neuronx_distributed_amd.models import PokepelConfig, build_model

    if (case, dtype) not in _models:
        cfg = pc.CASES[case]
        m = build_model("Pokepel", PokepelConfig.from_dict(cfg), dtype,
                        "cuda")
        m.load_checkpoint(pc.weights(cfg))
        _models[case, dtype] = m
    return _models[case, dtype]


def _prompt(case, n, seed=0):
    return pc.prompt(case, n, seed)


def _rms(x):
    return x.pow(2).mean(1).sqrt()


def _expected(case, tokens):
    """Logits, with the limit of every position in bf16."""
    key = case, tuple(tokens)
    if key not in _want:
        cfg = pc.CASES[case]
        w = pc.weights(cfg)
        want = po.forward(cfg, w, tokens)
        kept = po.norm, po.silu, po.sigmoid
        near = lambda f: lambda *a: f(*a).bfloat16().double()
        po.norm, po.silu, po.sigmoid = map(near, kept)
        try:
            rounded = po.forward(cfg, w, tokens)
        finally:
            po.norm, po.silu, po.sigmoid = kept
        want.limit = (4 * _rms(rounded - want) / want.pow(2).mean().sqrt()
                      ).clamp(min=LIMIT[torch.bfloat16])
        _want[key] = want
    return _want[key]


def _engine(case, dtype, max_tokens=1024, max_seqs=4, **kw):
    from neuronx_distributed_amd.inference import InferenceEngine

    return InferenceEngine(_model(case, dtype), max_tokens, max_seqs, **kw)


def _entry(*a):
    from neuronx_distributed_amd.inference import StepEntry

    return StepEntry(*a)


def _check(got, want, dtype, what):
    limit = getattr(want, "limit", None)     # a whole prompt's
    got, want = got.double().cpu(), want.double()
    assert torch.isfinite(got).all(), what
    if dtype == torch.float32 or limit is None:
        limit = torch.full((len(got),), LIMIT[dtype])
    err = _rms(got - want) / want.pow(2).mean().sqrt() / limit
    over = int((err > 1).sum())
    spare = max(1, len(err) // 50) if dtype == torch.bfloat16 else 0
    assert over <= spare and err.max() < 15, (
        what, over, err.max().item(), err.argmax().item())


def _feed(eng, rid, tokens, cuts):
    """One request alone; logits of every token."""
    out, at = [], 0
    for n in cuts:
        out.append(eng.step([_entry(rid, tokens[at:at + n], range(n))]))
        at += n
    assert at == len(tokens)
    eng.finish(rid)
    return torch.cat(out)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", list(pc.CASES))
def test_portions_and_decoding(case, dtype):
    T = 200
    toks = _prompt(case, T)
    want = _expected(case, toks)
    eng = _engine(case, dtype)
    for cuts in ([T], [2] * 100, [64, 64, 64, 8], [65, 1, 63, 2, 69],
                 [1] * T, [130] + [1] * 70, [3, 1, 1, 128, 2, 1, 64]):
        _check(_feed(eng, "a", toks, cuts), want, dtype, (case, cuts[:5]))
    assert eng.cache.free_pages == eng.cache.num_pages
    assert eng.cache.free_slots == 4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", ["mixed", "odd"])
def test_first_tokens(case, dtype):
    toks = _prompt(case, 9, seed=5)
    eng = _engine(case, dtype)
    for n in (1, 2, 3, 9):
        got = _feed(eng, n, toks[:n], [n])
        _check(got, _expected(case, toks[:n]), dtype, (case, n))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", ["mixed", "memories", "odd", "wide"])
def test_mixed_batches_reuse_pages_and_slots(case, dtype):
    """Six requests over four slots and a pool that holds about three:
    portions beside decoded tokens, requests left out of steps."""
    lens = [150, 33, 190, 1, 64, 97]
    toks = [_prompt(case, n, seed=i) for i, n in enumerate(lens)]
    eng = _engine(case, dtype, max_tokens=448)
    g = torch.Generator().manual_seed(3)
    at, got = [0] * 6, [[] for _ in lens]
    live, todo = [], list(range(6))
    used = {}
    for _ in range(2000):
        while todo and len(live) < 4 and sum(
                -(-lens[i] // 64) for i in live + todo[:1]) <= 7:
            live.append(todo.pop(0))
        if not live:
            break
        entries = []
        for i in live:
            r = int(torch.randint(0, 8, (1,), generator=g))
            n = min((0, 1, 1, 1, 2, 3, 17, 70)[r], lens[i] - at[i])
            if n:
                entries.append((i, n))
        if not entries:
            continue
        order = torch.randperm(len(entries), generator=g).tolist()
        entries = [entries[k] for k in order]
        res = eng.step([_entry(i, toks[i][at[i]:at[i] + n], range(n))
                        for i, n in entries])
        row = 0
        for i, n in entries:
            used.setdefault(eng.cache.requests[i].slot, set()).add(i)
            got[i].append(res[row:row + n])
            row += n
            at[i] += n
            if at[i] == lens[i]:
                eng.finish(i)
                live.remove(i)
    assert not todo and not live
    assert any(len(u) > 1 for u in used.values())
    for i in range(6):
        _check(torch.cat(got[i]), _expected(case, toks[i]), dtype, (case, i))


@pytest.mark.parametrize("dtype", DTYPES)
def test_wanted_places(dtype):
    """Logits come in the order of the entries and of their places; a step
    that wants nothing still advances the requests."""
    case = "mixed"
    a, b = _prompt(case, 40), _prompt(case, 25, seed=9)
    eng = _engine(case, dtype)
    assert eng.step([_entry("a", a[:30]), _entry("b", b[:1])]) is None
    got = eng.step([_entry("b", b[1:], [20, 3]), _entry("a", a[30:31], [0])])
    wa, wb = _expected(case, a), _expected(case, b)
    _check(got, torch.stack([wb[21], wb[4], wa[30]]), dtype, "order")
    assert eng.step([_entry("a", a[31:32])]) is None
    got = eng.step([_entry("a", a[32:], [7])])
    _check(got, wa[39:40], dtype, "after a silent step")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    """Decoding over many pages, then another request on the same pages and
    slot."""
    case, T = "mixed", 420
    toks = _prompt(case, T, seed=2)
    eng = _engine(case, dtype, max_tokens=448, max_seqs=1)
    got = _feed(eng, "x", toks, [3] + [1] * (T - 3))
    _check(got, _expected(case, toks), dtype, case)
    toks = _prompt(case, 100, seed=3)
    for cuts in ([50, 50], [1] * 100, [2, 98]):
        _check(_feed(eng, "y", toks, cuts), _expected(case, toks), dtype,
               cuts[:2])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", ["mixed", "wide"])
def test_prompts_over_several_chunks(case, dtype):
    T = 600
    toks = _prompt(case, T, seed=4)
    want = _expected(case, toks)
    eng = _engine(case, dtype, max_tokens=640, max_seqs=1)
    for cuts in ([T], [256, 344], [300, 2, 254, 1, 43], [511, 1, 88],
                 [513] + [1] * 87):
        _check(_feed(eng, "z", toks, cuts), want, dtype, (case, cuts[:4]))


def test_far_keys_show():
    """Changing the first token moves the last logits by far more than the
    limit, in a prompt and when decoding, and the engine follows."""
    case, dtype, T = "mixed", torch.float32, 300
    a = _prompt(case, T, seed=7)
    b = [(a[0] + 1) % pc.CASES[case]["vocab"]] + a[1:]
    wa, wb = _expected(case, a)[-20:], _expected(case, b)[-20:]
    moved = (wa - wb).pow(2).mean(1).sqrt() / wa.pow(2).mean().sqrt()
    assert moved.min() > 20 * LIMIT[dtype]
    eng = _engine(case, dtype)
    for toks, want in ((a, wa), (b, wb)):
        for cuts in ([T], [T - 20] + [1] * 20, [90, 90, 120]):
            _check(_feed(eng, 0, toks, cuts)[-20:], want, dtype, cuts[:2])


def test_graph_replays_equal_eager_steps():
    """Captured decode steps against eager ones, replay after replay, with
    eager work and synchronization between, and batches of 1..4 rows."""
    case, dtype = "mixed", torch.bfloat16
    toks = [_prompt(case, 60, seed=i) for i in range(4)]
    outs = []
    for graphs in (True, False):
        eng = _engine(case, dtype, use_graphs=graphs)
        res = []
        for i in range(4):
            eng.step([_entry(i, toks[i][:20 + i])])
        at = [20 + i for i in range(4)]
        for step in range(30):
            who = [i for i in range(4) if (step + i) % (i + 1) == 0]
            res.append(eng.step([_entry(i, [toks[i][at[i]]], [0])
                                 for i in who]))
            for i in who:
                at[i] += 1
            if step % 7 == 3:
                torch.cuda.synchronize()
                _ = (torch.ones(512, 512, device="cuda") @
                     torch.ones(512, 512, device="cuda")).sum().item()
        outs.append(res)
        assert bool(eng._graphs) == graphs
    # the number of workgroups that share a row, and so the order of sums,
    # may differ between the two
    for a, b in zip(*outs):
        _check(a, b.cpu(), dtype, "replay")


def test_refused_steps_change_nothing():
    from neuronx_distributed_amd.inference import CacheFull

    case, dtype = "mixed", torch.float32
    toks = _prompt(case, 70)
    eng = _engine(case, dtype, max_tokens=128, max_seqs=1)
    g1 = eng.step([_entry("a", toks[:30], range(30))])
    with pytest.raises(CacheFull):
        eng.step([_entry("b", [1], [0])])
    with pytest.raises(CacheFull):
        eng.step([_entry("a", [1] * 200, [0])])
    g2 = eng.step([_entry("a", toks[30:], range(40))])
    _check(torch.cat([g1, g2]), _expected(case, toks), dtype, "a")


def _greedy(case, prompt, n):
    cfg = pc.CASES[case]
    w, toks, margin = pc.weights(cfg), list(prompt), []
    for _ in range(n):
        top = po.forward(cfg, w, toks)[-1].topk(2)
        margin.append((top.values[0] - top.values[1]).item())
        toks.append(int(top.indices[0]))
    return toks[len(prompt):], min(margin)


@pytest.mark.parametrize("case", ["mixed", "odd"])
def test_greedy_generation(case, tmp_path):
    """generate(), the scheduler with small portions and few slots, and the
    command line give the oracle's greedy tokens."""
    from neuronx_distributed_amd.inference import generate, generate_ragged

    prompts = [_prompt(case, n, seed=20 + n) for n in (3, 70, 1, 41, 12)]
    want = [_greedy(case, p, 6) for p in prompts]
    assert min(m for _, m in want) > 1e-4       # no near ties
    want = [w for w, _ in want]
    m = _model(case, torch.float32)
    for kw in ({}, {"max_seqs": 2, "max_step_tokens": 9},
               {"max_step_tokens": 30, "use_graphs": False}):
        assert generate_ragged(m, prompts, 6, **kw) == want, kw
    x = torch.tensor([prompts[1], prompts[1]]).cuda()
    out = generate(m, x, max_new_tokens=6)
    assert out[:, 70:].tolist() == [want[1], want[1]]
    pc.save(pc.CASES[case], pc.weights(pc.CASES[case]), tmp_path)
    r = subprocess.run(
        [sys.executable, "-m", "neuronx_distributed_amd.scripts.generate",
         "--model", str(tmp_path), "--dtype", "float32",
         "--max-new-tokens", "6", "--max-seqs", "3"]
        + [a for p in prompts for a in ("--prompt", ",".join(map(str, p)))],
        capture_output=True, text=True, timeout=100, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-2000:]
    rows = [json.loads(l) for l in r.stdout.splitlines()
            if l.startswith("{")]
    assert [x["output"] for x in rows] == want


def test_sampled_generation_runs():
    from neuronx_distributed_amd.inference import generate_ragged
    from neuronx_distributed_amd.utils.sampling import Sampler

    case = "mixed"
    out = generate_ragged(_model(case, torch.bfloat16),
                          [_prompt(case, 5), _prompt(case, 9)], 8,
                          Sampler(do_sample=True, top_k=20, top_p=0.9))
    assert [len(o) for o in out] == [8, 8]
    assert all(0 <= t < pc.CASES[case]["vocab"] for o in out for t in o)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run(dtype, tmp_path):
    case = "mixed"
    cfg = pc.CASES[case]
    (tmp_path / "m").mkdir()
    (tmp_path / "out").mkdir()
    pc.save(cfg, pc.weights(cfg), tmp_path / "m")
    toks = [_prompt(case, 80, seed=i) for i in range(2)]
    steps = [
        {"entries": [{"id": "a", "tokens": toks[0][:50], "want": [49, 0]}],
         "end": []},
        {"entries": [{"id": "a", "tokens": toks[0][50:51], "want": []},
                     {"id": "b", "tokens": toks[1][:66], "want": []}],
         "end": []},
        {"entries": [{"id": "b", "tokens": toks[1][66:], "want": [13]},
                     {"id": "a", "tokens": toks[0][51:52], "want": [0]}],
         "end": ["b", "a"]},
    ]
    text = "".join(json.dumps({"step": i, **s}) + "\n"
                   for i, s in enumerate(steps))
    r = subprocess.run(
        [os.path.join(ROOT, "bin", "trace_run"), "--model",
         str(tmp_path / "m"), "--dtype", dtype, "--out",
         str(tmp_path / "out"), "--max-tokens", "256"],
        input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == \
        [f"done {i}" for i in range(3)]
    assert not (tmp_path / "out" / "1.f32").exists()
    w = [_expected(case, t) for t in toks]
    for i, rows in ((0, [w[0][49], w[0][0]]), (2, [w[1][79], w[0][51]])):
        raw = (tmp_path / "out" / f"{i}.f32").read_bytes()
        got = torch.frombuffer(bytearray(raw), dtype=torch.float32)
        _check(got.view(len(rows), -1), torch.stack(rows),
               getattr(torch, dtype), i)
