#!/usr/bin/env python3
"""Serving benchmark of the Voletar design beside Llama at equal layer sizes
(random weights, one MI355X):

    python bench.py --serving            kernels and whole models
    python bench.py --serving kernels    (or: models)

Kernels: time, roofline time (the larger of MFMA flops at 2.5 PFLOP/s and
bytes at 8 TB/s) and how far from it, for each serving kernel and the like
kernel that Llama runs.  Models: prefill and decode tokens/s.  Both sides are
timed in turn in one process; one JSON line per result.
"""

import json
import math
import time

import torch

PEAK_FLOPS, PEAK_BYTES = 2.5e15, 8.0e12


def _time(fns, reps=20, rounds=3):
    """Microseconds of each function, timed in turn, best of ``rounds``."""
    best = [math.inf] * len(fns)
    for f in fns:
        f()
        f()
    for _ in range(rounds):
        for i, f in enumerate(fns):
            a, b = (torch.cuda.Event(enable_timing=True) for _ in range(2))
            a.record()
            for _ in range(reps):
                f()
            b.record()
            torch.cuda.synchronize()
            best[i] = min(best[i], a.elapsed_time(b) * 1e3 / reps)
    return best


def _graphed(f):
    """Replay of f: times the kernels without their launch from Python."""
    f()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        f()
    return g.replay


def _report(name, us, flops, nbytes, like=None, **extra):
    roof = max(flops / PEAK_FLOPS, nbytes / PEAK_BYTES) * 1e6
    r = {"kernel": name, "us": round(us, 1), "roofline_us": round(roof, 2),
         "times_roofline": round(us / roof, 2), **extra}
    if like:
        lname, lus, lflops, lbytes = like
        lroof = max(lflops / PEAK_FLOPS, lbytes / PEAK_BYTES) * 1e6
        r["like"] = {"kernel": lname, "us": round(lus, 1),
                     "roofline_us": round(lroof, 2),
                     "times_roofline": round(lus / lroof, 2)}
        r["distance_ratio"] = round((us / roof) / (lus / lroof), 2)
    print(json.dumps(r), flush=True)


def _bf(*shape):
    return torch.randn(*shape, device="cuda", dtype=torch.float32).bfloat16()


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device="cuda")


def bench_kernels():
    from neuronx_distributed_amd import ops
    from neuronx_distributed_amd.ops import serving as sv

    dev = dict(device="cuda")
    # -- attention over prompts ---------------------------------------------
    H, G, D = 32, 8, 128
    for T, W in ((4096, 4096), (8192, 4096), (8192, 1024)):
        p = _bf(T, (H + 2 * G) * D)
        q, k, v = p[:, :H * D], p[:, H * D:(H + G) * D], p[:, (H + G) * D:]
        pages = T // 64
        kc = torch.zeros(pages, G, 64, D, dtype=torch.bfloat16, **dev)
        vc = torch.zeros_like(kc)
        bt = torch.randperm(pages).int().cuda().view(1, -1)
        pos = torch.arange(T, dtype=torch.int32, **dev)
        seq = torch.zeros(T, dtype=torch.int32, **dev)
        tiles = _i32([(0, s, 128, s) for s in range(0, T, 128)])
        fq, fk, fv = (t.reshape(1, T, -1, D).transpose(1, 2).contiguous()
                      for t in (q, k, v))
        win = W if W < T else None
        us, lus = _time([
            _graphed(lambda: sv.attn_portions(
                q, k, v, kc, vc, pos, seq, bt, tiles, H, D ** -0.5, W, 64)),
            _graphed(lambda: ops.flash_attn(fq, fk, fv, True, None,
                                            win or 0))])
        pairs = sum(min(i + 1, W + min(64, max(0, i + 1 - W)))
                    for i in range(T))
        lpairs = sum(min(i + 1, W) for i in range(T))
        io = 2 * T * (2 * H + 2 * G) * D
        _report("attn_portions (append + tiles)", us, 4 * pairs * H * D,
                io + 4 * T * G * D,
                ("flash_attn", lus, 4 * lpairs * H * D, io),
                tokens=T, window=W)
    # -- attention of single tokens -----------------------------------------
    for B, ctx in ((1, 4096), (32, 1024), (32, 4096), (128, 4096)):
        Smax = ctx + 64
        p = _bf(B, (H + 2 * G) * D)
        q, k, v = p[:, :H * D], p[:, H * D:(H + G) * D], p[:, (H + G) * D:]
        n = Smax // 64
        kc = torch.zeros(B * n, G, 64, D, dtype=torch.bfloat16, **dev)
        vc = torch.zeros_like(kc)
        bt = torch.randperm(B * n).int().cuda().view(B, n)
        pos = torch.full((B,), ctx, dtype=torch.int32, **dev)
        seq = torch.arange(B, dtype=torch.int32, **dev)
        lk = torch.zeros(B, G, Smax, D, dtype=torch.bfloat16, **dev)
        lv = torch.zeros_like(lk)
        cos = torch.ones(Smax, D // 2, **dev)
        sin = torch.zeros(Smax, D // 2, **dev)
        pt = torch.tensor([ctx], dtype=torch.int64, **dev)
        us, lus = _time([
            _graphed(lambda: sv.attn_rows(
                q, k, v, kc, vc, pos, seq, bt, H, D ** -0.5, 4096, 64,
                max_keys=Smax)),
            _graphed(lambda: ops.decode_attn_step(
                q, k, v, lk, lv, cos, sin, pt, H, G, D ** -0.5))])
        nb = 4 * B * G * (ctx + 1) * D + 4 * B * H * D
        fl = 4 * B * H * (ctx + 1) * D
        _report("attn_rows", us, fl, nb, ("decode_attn_step", lus, fl, nb),
                batch=B, context=ctx)
    # -- matrix memories -----------------------------------------------------
    for gated, (H2, D2, E2) in ((False, (32, 128, 128)),
                                (True, (16, 128, 256)),
                                (True, (8, 256, 512))):
        for B, T in ((1, 4096), (4, 4096), (1, 1), (32, 1), (128, 1)):
            n = 2 * H2 * D2 + H2 * E2
            p = _bf(B * T, n + H2 * E2)
            q, k = p[:, :H2 * D2], p[:, H2 * D2:2 * H2 * D2]
            v = p[:, 2 * H2 * D2:n]
            nt = (E2 + 31) // 32
            S = torch.zeros(B, H2, D2, E2, **dev)
            nn = torch.zeros(B, H2, nt, D2, **dev)
            m = torch.zeros(B, H2, nt, **dev)
            ctx = 64 if T == 1 else 0
            seg = _i32([(b, b * T, T, ctx) for b in range(B)])
            if gated:
                b0 = torch.zeros(H2, dtype=torch.bfloat16, **dev)
                gate = sv.ExpGate(torch.randn(B * T, 2 * H2, **dev), b0,
                                  b0 + 3, 15.0, D2 ** -0.5)
            else:
                gate = sv.decay_gate([0.99] * H2, "cuda")
            rows, first = sv.chunk_table(seg.tolist())
            tab = (_i32(rows), _i32(first)) if T > 1 else ()
            (us,) = _time([_graphed(lambda: sv.memory_mix(
                q, k, v, gate, S, nn, m, seg, H2, *tab))])
            io = 2 * B * T * (n + H2 * E2) + \
                (8 if ctx else 4) * B * H2 * D2 * E2
            # chunked: scores, weighted values, state in and out
            C = 64 if T > 1 else 1
            fl = 2 * B * T * H2 * (C / 2 * (D2 + E2) + 2 * D2 * E2)
            # the same with every product of a 32-bit operand at its MFMA
            # cost, three bf16 products
            f3 = 2 * B * T * H2 * (C / 2 * (D2 + 3 * E2) + 6 * D2 * E2)
            extra = {"roofline_32bit_us": round(
                max(f3 / PEAK_FLOPS, io / PEAK_BYTES) * 1e6, 2)} \
                if T > 1 else {}
            _report("memory_" + ("chunks" if T > 1 else "steps"), us, fl, io,
                    gated=gated, heads=H2, dim=D2, vdim=E2, batch=B,
                    tokens=T, **extra)
    # -- norms and pointwise ---------------------------------------------------
    for T in (32, 4096):
        Wd, F = 4096, 14336
        x = torch.randn(T, Wd, **dev)
        xb, d, d2 = _bf(T, Wd), _bf(T, Wd), _bf(T, Wd)
        w = _bf(Wd)
        gt = _bf(T, 2 * Wd)
        u, gu = _bf(T, F), _bf(T, 2 * F)
        t = _time([
            _graphed(lambda: sv.residual_norm(x, sv.Pending(d), 1e-6, w)),
            _graphed(lambda: ops.add_rmsnorm(xb, d, w, 1e-6)),
            _graphed(lambda: sv.residual_norm(
                x, sv.Pending(d, d2, w, w, 0.5), 1e-6, w)),
            _graphed(lambda: sv.gated_norm(d, w, gt[:, Wd:], Wd, 1e-6)),
            _graphed(lambda: sv.gated_norm(d, w, gt[:, Wd:], 256, 1e-6)),
            _graphed(lambda: sv.relu_squared_(u)),
            _graphed(lambda: ops.swiglu(gu))])
        n = T * Wd
        like = ("add_rmsnorm", t[1], 0, 8 * n)
        _report("residual_norm", t[0], 0, 12 * n, like, rows=T)
        _report("residual_norm (two branches)", t[2], 0, 14 * n, like, rows=T)
        _report("gated_norm (all heads)", t[3], 0, 6 * n, like, rows=T)
        _report("gated_norm (per head)", t[4], 0, 6 * n, like, rows=T)
        _report("relu_squared", t[5], 0, 4 * T * F,
                ("swiglu", t[6], 0, 6 * T * F), rows=T)


def bench_models(layers=None):
    from neuronx_distributed_amd.inference import (InferenceEngine, StepEntry,
                                                   single_process_groups)
    from neuronx_distributed_amd.inference.decode_graph import GraphDecoder
    from neuronx_distributed_amd.inference.kv_cache import build_kv_caches
    from neuronx_distributed_amd.models import (build_model, get_config,
                                                get_voletar_config)

    single_process_groups()
    torch.manual_seed(0)
    vcfg = get_voletar_config("voletar-bench")
    runs = len(vcfg.schedule())
    vol = build_model("Voletar", vcfg, torch.bfloat16, "cuda")
    lcfg = get_config("mistral-7b", num_hidden_layers=runs,
                      max_position_embeddings=16384, sliding_window=None)
    lla = build_model("LlamaForCausalLM", lcfg, torch.bfloat16, "cuda")
    size = lambda m: sum(p.numel() for p in m.parameters()) / 1e9
    print(json.dumps({"voletar_b_params": round(size(vol), 2),
                      "llama_b_params": round(size(lla), 2),
                      "layer_runs": runs, "data": "random weights"}),
          flush=True)

    # prefill; both sides compute the last token's logits only for Voletar,
    # all tokens' for Llama (its forward has no selection): the head is
    # subtracted from Llama by running its decoder stack alone
    for B, T in ((1, 2048), (1, 4096), (4, 4096)):
        toks = torch.randint(0, 32000, (B, T))
        x = toks.cuda()
        rows = toks.tolist()
        eng = InferenceEngine(vol, max_tokens=B * T, max_seqs=B)
        caches = build_kv_caches(runs, B, lcfg.num_key_value_heads, T,
                                 lcfg.head_dim, device=x.device)

        def run_v():
            eng.step([StepEntry(b, rows[b], [T - 1]) for b in range(B)])
            for b in range(B):
                eng.finish(b)

        def run_l():
            with torch.no_grad():
                h = lla.model(x, 0, caches)
                lla.lm_head(h[:, -1])

        best = [math.inf, math.inf]
        for _ in range(4):
            for i, f in enumerate((run_v, run_l)):
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                f()
                torch.cuda.synchronize()
                best[i] = min(best[i], time.perf_counter() - t0)
        print(json.dumps({
            "prefill": {"batch": B, "tokens": T},
            "voletar_tokens_per_s": round(B * T / best[0]),
            "llama_tokens_per_s": round(B * T / best[1])}), flush=True)
        del eng, caches
        torch.cuda.empty_cache()

    # decode: graph replays with greedy feedback
    for B, ctx in ((1, 2048), (32, 2048), (128, 2048)):
        steps = 24
        x = torch.randint(0, 32000, (B, ctx))
        eng = InferenceEngine(vol, max_tokens=B * (ctx + 64), max_seqs=B,
                              max_context=ctx + 64)
        rows = x.tolist()
        for b in range(B):
            eng.step([StepEntry(b, rows[b])])
        tok = [1] * B

        def step_v(tok):
            lg = eng.step([StepEntry(b, [tok[b]], [0]) for b in range(B)])
            return lg.argmax(-1).tolist()

        caches = build_kv_caches(runs, B, lcfg.num_key_value_heads, ctx + 64,
                                 lcfg.head_dim, device="cuda")
        dec = GraphDecoder(lla, caches, start_pos=ctx, batch=B,
                           device=torch.device("cuda"))
        with torch.no_grad():
            dec.capture()
        tl = torch.ones(B, dtype=torch.long, device="cuda")
        best = [math.inf, math.inf]
        for _ in range(3):
            for side in (0, 1):
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                for _ in range(steps // 3):
                    if side == 0:
                        tok = step_v(tok)
                    else:
                        tl = dec.step(tl)[:, -1].argmax(-1)
                        tl.tolist()
                torch.cuda.synchronize()
                best[side] = min(best[side],
                                 (time.perf_counter() - t0) / (steps // 3))
        print(json.dumps({
            "decode": {"batch": B, "context": ctx},
            "voletar_ms": round(best[0] * 1e3, 3),
            "llama_ms": round(best[1] * 1e3, 3),
            "voletar_tokens_per_s": round(B / best[0]),
            "llama_tokens_per_s": round(B / best[1])}), flush=True)
        del eng, caches, dec
        torch.cuda.empty_cache()


def main(what="all"):
    torch.cuda.set_device(0)
    if what in ("all", "kernels"):
        bench_kernels()
    if what in ("all", "models"):
        bench_models()


if __name__ == "__main__":
    import sys

    main(*sys.argv[1:2])
