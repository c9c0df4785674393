#!/usr/bin/env python3
"""Serving benchmark of a design beside its closest relative at equal layer
sizes (random weights, one MI355X): Voletar beside Llama, Nesilorn beside
Mixtral, Sutuvik and Pokepel beside Nesilorn (their kernels beside those of
Voletar and Nesilorn).

    python bench.py --serving                          all of it
    python bench.py --serving kernels                  (or: models)
    python bench.py --serving kernels --design nesilorn

Kernels: time, roofline time (the larger of MFMA flops at 2.5 PFLOP/s and
bytes at 8 TB/s) and how far from it, for each serving kernel and the like
kernel that the relative runs.  Models: prefill and decode tokens/s.  Both
sides are timed in turn in one process; one JSON line per result.
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


# ---------------------------------------------------------------------------
# Nesilorn beside Mixtral
# ---------------------------------------------------------------------------

def _kernel_us(f, name, reps=10):
    """Device microseconds a call of f spends in kernels called ``name``: for
    calls that read the device from the host and cannot be captured."""
    from torch.profiler import ProfilerActivity, profile

    f()
    torch.cuda.synchronize()
    with profile(activities=[ProfilerActivity.CUDA,
                             ProfilerActivity.CPU]) as prof:
        for _ in range(reps):
            f()
        torch.cuda.synchronize()
    return sum(e.self_device_time_total for e in prof.key_averages()
               if name in e.key) / reps


def _latent_case(sv, B, T, ctx, H, D, P, E, R):
    """A packed step of B requests with T new tokens each at context ctx."""
    from types import SimpleNamespace

    n = -(-(ctx + T) // 64)
    bt = torch.randperm(B * n).int().view(B, n)
    b = SimpleNamespace(
        block_table=bt.cuda(), max_keys=ctx + T,
        pos=_i32(list(range(ctx, ctx + T)) * B),
        seq=_i32([r for r in range(B) for _ in range(T)]),
        portion_tokens=B * T if T > 1 else 0, spans={})
    if T > 1:
        b.tiles = _i32([(r, r * T + s, 128, ctx + s) for r in range(B)
                        for s in range(0, T, 128)])
    w = sv.LatentWeights(
        _bf(R), (torch.randn(H, R, D, device="cuda") * R ** -0.5).bfloat16(),
        (torch.randn(H * (D + E), R, device="cuda") * R ** -0.5).bfloat16(),
        sv.rotary_frequencies(1e4, P, "cuda"))
    cache = _bf(B * n, 64, R + P)
    sizes = (H * (D + P), R + P, H * E)
    p = _bf(B * T, sum(sizes))
    q, kv, g = p.split(sizes, 1)
    return b, w, cache, q, kv, g


def bench_latent_kernels():
    from neuronx_distributed_amd import ops
    from neuronx_distributed_amd.ops import serving as sv

    dev = dict(device="cuda")
    H, D, P, E, R, G, LD = 32, 128, 64, 128, 512, 8, 128
    scale = (D + P) ** -0.5
    # -- prompts -------------------------------------------------------------
    for T, W in ((4096, 4096), (8192, 4096), (8192, 1024)):
        b, w, cache, q, kv, g = _latent_case(sv, 1, T, 0, H, D, P, E, R)
        pages, table = sv.key_spans([(0, 0, T, 0)], b.block_table.tolist(), W)
        b.spans = {W: sv.KeySpans(_i32(pages), _i32(table))}
        out = torch.empty(T, H * E, dtype=torch.bfloat16, **dev)
        fq, fk, fv = (_bf(1, h, T, LD) for h in (H, G, G))
        win = W if W < T else 0
        kve = _bf(T, H * (D + E))
        ws = _bf(T, R + P)
        us, tus, lus = _time([
            _graphed(lambda: sv.latent_attention(
                q, kv, g, b, cache, w, H, D, E, scale, 1e-5, W)),
            _graphed(lambda: sv.expanded_attention(
                q, g, kve, ws, b.tiles, b.spans[W], H, D, E, scale, W, out)),
            _graphed(lambda: ops.flash_attn(fq, fk, fv, True, None, win))])
        pairs = sum(min(i + 1, W) for i in range(T))
        lio = 2 * T * (2 * H + 2 * G) * LD
        like = ("flash_attn", lus, 4 * pairs * H * LD, lio)
        fl = 2 * pairs * H * (D + P + E)
        io = 2 * T * (H * (D + P + 2 * E) + R + P)
        _report("latent_attention (append, gather, expand, tiles)", us,
                fl + 2 * T * R * H * (D + E), io, like, tokens=T, window=W)
        _report("attn_tiles on expanded keys", tus, fl,
                io + 2 * T * H * (D + E), like, tokens=T, window=W)
    # -- single tokens ---------------------------------------------------------
    for B, ctx in ((1, 4096), (32, 1024), (32, 4096), (128, 4096)):
        b, w, cache, q, kv, g = _latent_case(sv, B, 1, ctx, H, D, P, E, R)
        ql = _bf(B, H * (R + P))
        Smax = ctx + 64
        lq, lk, lv = _bf(B, H * LD), _bf(B, G * LD), _bf(B, G * LD)
        kc = torch.zeros(B, G, Smax, LD, dtype=torch.bfloat16, **dev)
        vc = torch.zeros_like(kc)
        cos = torch.ones(Smax, LD // 2, **dev)
        pt = torch.tensor([ctx], dtype=torch.int64, **dev)
        lat = _bf(B, H * R)
        out = _bf(B, H * E)
        wv = w.expand[H * D:].view(H, E, R)
        wl = _bf(E * H, R)
        t = _time([
            _graphed(lambda: sv.latent_attention(
                q, kv, g, b, cache, w, H, D, E, scale, 1e-5, 4096)),
            _graphed(lambda: sv.latent_rows(
                ql, cache, R, b.pos, b.seq, b.block_table, H, scale, 4096,
                ctx + 1)),
            _graphed(lambda: ops.decode_attn_step(
                lq, lk, lv, kc, vc, cos, cos, pt, H, G, LD ** -0.5)),
            _graphed(lambda: sv.head_linear(q, D + P, w.absorb, ql, R + P)),
            _graphed(lambda: sv.head_linear(lat, R, wv, out, E, g)),
            _graphed(lambda: torch.mm(lat[:, :R], wl.t())),
            _graphed(lambda: sv.latent_append(
                q, D, D + P, ql, R, R + P, kv, w, cache, b.pos, b.seq,
                b.block_table, H, 1e-5))])
        lb = 4 * B * G * (ctx + 1) * LD + 4 * B * H * LD
        like = ("decode_attn_step", t[2], 4 * B * H * (ctx + 1) * LD, lb)
        cb = 2 * B * min(ctx + 1, 4096) * (R + P)
        fl = 2 * B * H * min(ctx + 1, 4096) * (2 * R + P)
        wb = 2 * H * (D + E) * R
        _report("latent_attention (append, absorb, rows, values)", t[0],
                fl + 2 * B * H * R * (D + E),
                cb + wb + 2 * B * H * (D + P + 2 * E), like, batch=B,
                context=ctx)
        _report("latent_rows", t[1], fl, cb + 2 * B * H * (2 * R + P), like,
                batch=B, context=ctx)
        mm = ("mm of the same weights", t[5], 2 * B * H * E * R,
              2 * H * E * R + 2 * B * (R + H * E))
        _report("head_linear (absorb)", t[3], 2 * B * H * D * R,
                2 * H * D * R + 2 * B * H * (D + R), mm, batch=B)
        _report("head_linear (values, gate)", t[4], 2 * B * H * E * R,
                2 * H * E * R + 2 * B * H * (2 * E + R), mm, batch=B)
        _report("latent_append", t[6], 0, 4 * B * (H * P + R + P), batch=B)
    # -- experts ---------------------------------------------------------------
    for (Wd, ff, n, top) in ((4096, 14336, 8, 2), (2048, 1408, 64, 6)):
        gu, down = (torch.randn(n, a, c, device="cuda",
                                dtype=torch.bfloat16) * c ** -0.5
                    for a, c in ((2 * ff, Wd), (Wd, ff)))
        bias = _bf(n)
        lgu = gu.transpose(1, 2).contiguous()
        ldn = down.transpose(1, 2).contiguous()
        for T in (1, 32, 128, 512, 4096, 16384):
            x, z = _bf(T, Wd), torch.randn(T, n, **dev)
            how = sv.moe_kernel(T * top, n)
            plan = sv.moe_plan(z, bias, top, how)
            act = sv.moe_gemm(x, gu, plan, True, 1.702, 7.0, 1.0)
            hit = int(plan.idx.unique().numel())
            idx = plan.idx.long()
            fns = [_graphed(lambda: sv.moe_mlp(x, z, bias, gu, down, top,
                                               1.702, 7.0, 1.0)),
                   _graphed(lambda: sv.moe_plan(z, bias, top, how)),
                   _graphed(lambda: sv.moe_gemm(x, gu, plan, True, 1.702,
                                                7.0, 1.0)),
                   _graphed(lambda: sv.moe_gemm(act, down, plan, False))]
            if T <= 512:
                aff = torch.zeros(T, n, **dev).scatter_(1, idx, 0.5)
                t = _time(fns)
                lus = _kernel_us(lambda: ops.moe_decode_glu(
                    x, lgu, ldn, aff, idx), "moe_")
                name = "moe_decode_glu, its kernels"
            else:
                rows = plan.order.long() // top
                xs = x[rows].contiguous()
                offs = torch.bincount(idx.flatten(), minlength=n).cumsum(
                    0).int()

                def grouped():
                    a = ops.swiglu(torch._grouped_mm(xs, lgu, offs=offs))
                    return torch._grouped_mm(a, ldn, offs=offs)
                try:
                    t = _time(fns + [grouped])
                    lus = t[4]
                except RuntimeError as e:
                    print(json.dumps({"skipped": "_grouped_mm",
                                      "why": str(e)[:100]}), flush=True)
                    t, lus = _time(fns), None
                name = "grouped_mm, swiglu, grouped_mm"
            fl = 6 * T * top * Wd * ff
            io = 6 * hit * Wd * ff + 2 * T * Wd * (1 + top)
            kw = dict(tokens=T, width=Wd, ff=ff, experts=n, top=top)
            _report("moe_mlp (plan, gate/up, down)", t[0], fl, io,
                    lus and (name, lus, fl, io), **kw)
            _report("moe_gemm (gate/up)", t[2], fl * 2 / 3,
                    4 * hit * Wd * ff + 2 * T * (Wd + top * ff), **kw)
            _report("moe_gemm (down)", t[3], fl / 3,
                    2 * hit * Wd * ff + 2 * T * top * (Wd + ff), **kw)
            _report("moe_plan", t[1], 0, 4 * T * n + 12 * T * top, **kw)
        del gu, down, lgu, ldn
        torch.cuda.empty_cache()
    # -- norms and pointwise -----------------------------------------------------
    for T in (32, 4096):
        Wd, F, top = 4096, 14336, 2
        x, xb, d = torch.randn(T, Wd, **dev), _bf(T, Wd), _bf(T, Wd)
        d2, coef, w = _bf(T * top, Wd), torch.rand(T, top, **dev), _bf(Wd)
        u, gu = _bf(T, F), _bf(T, 2 * F)
        kw = dict(w1=w, centred=True)
        t = _time([
            _graphed(lambda: sv.residual_norm(
                x, sv.Pending(d, **kw), 1e-6, copy=True,
                dtype=torch.bfloat16)),
            _graphed(lambda: sv.residual_norm(
                x, sv.Pending(d2, coef=coef, **kw), 1e-6, copy=True,
                dtype=torch.bfloat16)),
            _graphed(lambda: ops.add_rmsnorm(xb, d, w, 1e-6)),
            _graphed(lambda: sv.gelu_tanh_(u)),
            _graphed(lambda: ops.swiglu(gu))])
        n = T * Wd
        like = ("add_rmsnorm", t[2], 0, 8 * n)
        _report("residual_norm (output norm)", t[0], 0, 12 * n, like, rows=T)
        _report("residual_norm (experts' sum, output norm)", t[1], 0,
                (10 + 2 * top) * n, like, rows=T)
        _report("gelu_tanh", t[3], 0, 4 * T * F,
                ("swiglu", t[4], 0, 6 * T * F), rows=T)


def bench_latent_models():
    import os

    from neuronx_distributed_amd.inference import (InferenceEngine, StepEntry,
                                                   single_process_groups)
    from neuronx_distributed_amd.inference.kv_cache import build_kv_caches
    from neuronx_distributed_amd.models import (build_model,
                                                get_nesilorn_config)
    from neuronx_distributed_amd.models.mixtral import (MixtralForCausalLM,
                                                        get_moe_config)

    single_process_groups()
    torch.manual_seed(0)
    cfg = get_nesilorn_config("nesilorn-bench")
    n = len(cfg.layers)
    nes = build_model("Nesilorn", cfg, torch.bfloat16, "cuda")
    mcfg = get_moe_config("mixtral-8x7b", num_hidden_layers=n,
                          max_position_embeddings=16384, capacity_factor=0.0)
    os.environ["NXDA_FAST_INIT"] = "1"
    torch.set_default_dtype(torch.bfloat16)
    try:
        with torch.device("cuda"):
            mix = MixtralForCausalLM(mcfg).eval()
    finally:
        torch.set_default_dtype(torch.float32)
        del os.environ["NXDA_FAST_INIT"]
    size = lambda m: sum(p.numel() for p in m.parameters()) / 1e9
    print(json.dumps({"nesilorn_b_params": round(size(nes), 2),
                      "mixtral_b_params": round(size(mix), 2),
                      "layers": n, "data": "random weights"}), flush=True)

    def caches_for(B, T):
        return build_kv_caches(n, B, mcfg.num_key_value_heads, T,
                               mcfg.head_dim, device=torch.device("cuda"))

    # logits of the last token on both sides
    for B, T in ((1, 2048), (1, 4096), (4, 4096)):
        toks = torch.randint(0, 32000, (B, T))
        x, rows = toks.cuda(), toks.tolist()
        eng = InferenceEngine(nes, max_tokens=B * T, max_seqs=B)
        caches = caches_for(B, T)

        def run_n():
            eng.step([StepEntry(b, rows[b], [T - 1]) for b in range(B)])
            for b in range(B):
                eng.finish(b)

        def run_m():
            with torch.no_grad():
                h, _ = mix.model(x, 0, caches)
                mix.lm_head(h[:, -1])

        best = [math.inf, math.inf]
        for _ in range(4):
            for i, f in enumerate((run_n, run_m)):
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                f()
                torch.cuda.synchronize()
                best[i] = min(best[i], time.perf_counter() - t0)
        print(json.dumps({
            "prefill": {"batch": B, "tokens": T},
            "nesilorn_tokens_per_s": round(B * T / best[0]),
            "mixtral_tokens_per_s": round(B * T / best[1])}), flush=True)
        del eng, caches
        torch.cuda.empty_cache()

    # decode with greedy feedback: the engine replays a graph; Mixtral runs
    # step by step, since its routing reads counts on the host
    for B, ctx in ((1, 2048), (32, 2048), (128, 2048)):
        steps = 8
        rows = torch.randint(0, 32000, (B, ctx)).tolist()
        eng = InferenceEngine(nes, max_tokens=B * (ctx + 64), max_seqs=B,
                              max_context=ctx + 64)
        for b in range(B):
            eng.step([StepEntry(b, rows[b])])
        tok = [1] * B

        def step_n(tok):
            lg = eng.step([StepEntry(b, [tok[b]], [0]) for b in range(B)])
            return lg.argmax(-1).tolist()

        caches = caches_for(B, ctx + 64)
        tl, at = torch.ones(B, 1, dtype=torch.long, device="cuda"), ctx
        tok = step_n(tok)
        best = [math.inf, math.inf]
        for _ in range(3):
            for side in (0, 1):
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                for _ in range(steps):
                    if side == 0:
                        tok = step_n(tok)
                    else:
                        with torch.no_grad():
                            lg = mix(tl, pos_offset=torch.tensor(
                                [at], device="cuda"), kv_caches=caches)
                        tl = lg[:, -1].argmax(-1, keepdim=True)
                        tl.tolist()
                        at += 1
                torch.cuda.synchronize()
                best[side] = min(best[side],
                                 (time.perf_counter() - t0) / steps)
        print(json.dumps({
            "decode": {"batch": B, "context": ctx},
            "nesilorn_ms": round(best[0] * 1e3, 3),
            "mixtral_ms": round(best[1] * 1e3, 3),
            "nesilorn_tokens_per_s": round(B / best[0]),
            "mixtral_tokens_per_s": round(B / best[1])}), flush=True)
        del eng, caches
        torch.cuda.empty_cache()


# ---------------------------------------------------------------------------
# Sutuvik beside Nesilorn and Voletar
# ---------------------------------------------------------------------------

def bench_state_kernels():
    from types import SimpleNamespace

    from neuronx_distributed_amd.models.mixers import alibi_slopes
    from neuronx_distributed_amd.ops import serving as sv

    dev = dict(device="cuda")
    bf = torch.bfloat16
    # -- timed memories beside decayed ones of half the state ----------------
    H, G, N, P, taps = 128, 8, 128, 64, 4
    LH, LD = 32, 128
    inner, gn = H * P, G * N
    C = inner + 2 * gn
    w, b = _bf(taps, C), _bf(C)
    small = [_bf(H) for _ in range(3)]
    like_gate = sv.decay_gate([0.99] * LH, "cuda")
    for B, T in ((1, 4096), (4, 4096), (1, 1), (32, 1), (128, 1)):
        n = B * T
        proj = _bf(n, inner + C)
        z, xbc = proj[:, :inner], proj[:, inner:]
        step = torch.randn(n, H, **dev)
        S = torch.zeros(B, H, N, P, **dev)
        ring = torch.zeros(B, taps, C, dtype=bf, **dev)
        conv = sv.ShortConv(w, ring, b)
        ctx = 64 if T == 1 else 0
        seg = _i32([(i, i * T, T, ctx) for i in range(B)])
        rows, first = sv.chunk_table(seg.tolist())
        tab = (_i32(rows), _i32(first)) if T > 1 else ()
        x = sv.short_conv(xbc, conv, seg, _i32(rows), silu=True) \
            if T > 1 else xbc
        v, k, q = x.split((inner, gn, gn), 1)
        gate = sv.TimeGate(step, *small, z, None if T > 1 else conv)
        lp = _bf(n, 3 * LH * LD)
        lq, lk, lv = lp.split(LH * LD, 1)
        LS = torch.zeros(B, LH, LD, LD, **dev)
        us, lus = _time([
            _graphed(lambda: sv.memory_mix(q, k, v, gate, S, None, None, seg,
                                           H, *tab)),
            _graphed(lambda: sv.memory_mix(lq, lk, lv, like_gate, LS, None,
                                           None, seg, LH, *tab))])
        cs = 64 if T > 1 else 1
        state = 8 if ctx else 4

        def cost(h, g, d, e, extra):
            return (2 * n * h * (cs / 2 * (d + e) + 2 * d * e),
                    2 * n * (2 * g * d + (2 + extra) * h * e)
                    + state * B * h * d * e)

        fl, io = cost(H, G, N, P, 1)
        io += 4 * n * H
        f3 = 2 * n * H * (cs / 2 * (N + 3 * P) + 6 * N * P)
        extra = {"roofline_32bit_us": round(
            max(f3 / PEAK_FLOPS, io / PEAK_BYTES) * 1e6, 2)} if T > 1 else {}
        if T == 1:
            io += 2 * n * (taps + 1) * C
        _report("memory_" + ("chunks" if T > 1 else "steps, convolution"), us,
                fl, io, ("decayed memory", lus, *cost(LH, LH, LD, LD, 0)),
                batch=B, tokens=T, heads=H, state=N, vdim=P, **extra)
    # -- attention -------------------------------------------------------------
    H, G, D = 32, 8, 128
    sizes = (H * D, G * D, G * D, H)
    slope = torch.tensor(alibi_slopes(H), **dev)
    freq = sv.rotary_frequencies(5e5, D, "cuda")
    nw, hw = _bf(D), _bf(H)
    kinds = {
        "bias, sink, gate": (
            sv.QkvPrep(norm=True, q_norm=nw, k_norm=nw, eps=1e-5,
                       temp_coef=0.1, temp_every=8192),
            lambda g: sv.ScoreMod(slope=slope, sink=hw, gate=g)),
        "rotation, cap, sink": (
            sv.QkvPrep(freq=freq, norm=True, eps=1e-5),
            lambda g: sv.ScoreMod(temp=hw, cap=50.0, sink=hw))}
    for B, T, ctx in ((1, 4096, 0), (1, 8192, 0), (1, 1, 4096), (32, 1, 1024),
                      (32, 1, 4096), (128, 1, 4096)):
        p = _bf(B * T, sum(sizes))
        q, k, v, g = p.split(sizes, 1)
        n = -(-(ctx + T) // 64)
        kc = torch.zeros(B * n, G, 64, D, dtype=bf, **dev)
        vc = torch.zeros_like(kc)
        batch = SimpleNamespace(
            block_table=torch.randperm(B * n).int().cuda().view(B, n),
            max_keys=ctx + T, pos=_i32(list(range(ctx, ctx + T)) * B),
            seq=_i32([r for r in range(B) for _ in range(T)]),
            portion_tokens=B * T if T > 1 else 0,
            tiles=_i32([(r, r * T + s, 128, ctx + s) for r in range(B)
                        for s in range(0, T, 128)] if T > 1 else []))
        pairs = B * sum(ctx + i + 1 for i in range(T))
        fl = 4 * pairs * H * D
        io = 2 * B * T * (2 * H + 2 * G) * D + \
            (4 * B * G * ctx * D if T == 1 else 0)
        for name, (prep, mod) in kinds.items():
            prep.first, prep.mix = v.clone(), nw[:1]
            at = (batch.pos, batch.seq, batch.block_table)
            us, pus, lus, aus = _time([
                _graphed(lambda: sv.ragged_attention(
                    q, k, v, batch, (kc, vc), H, D ** -0.5, prep=prep,
                    mod=mod(g))),
                _graphed(lambda: sv.qkv_append(q, k, v, kc, vc, *at, H, prep)),
                _graphed(lambda: sv.ragged_attention(
                    q, k, v, batch, (kc, vc), H, D ** -0.5)),
                _graphed(lambda: sv.kv_append(k, v, kc, vc, *at))])
            _report(f"attention ({name})", us, fl, io,
                    ("plain attention", lus, fl, io), batch=B, tokens=T,
                    context=ctx)
            _report(f"qkv_append ({name})", pus, 0,
                    2 * B * T * (2 * H + 5 * G) * D,
                    ("kv_append", aus, 0, 8 * B * T * G * D), batch=B,
                    tokens=T)
    # -- norms, convolutions, routing -------------------------------------------
    W = 4096
    for B, T in ((32, 1), (1, 4096)):
        n, top = B * T, 2
        x, d, wn = torch.randn(n, W, **dev), _bf(n, W), _bf(W)
        d2, coef = _bf(n * top, W), torch.rand(n, top, **dev)
        cw = sv.ShortConv(_bf(4, W), torch.zeros(B, 4, W, dtype=bf, **dev))
        seg = _i32([(i, i * T, T, 64 if T == 1 else 0) for i in range(B)])
        rows, _ = sv.chunk_table(seg.tolist())
        batch = SimpleNamespace(portion_tokens=n if T > 1 else 0,
                                portions=seg, chunks=_i32(rows),
                                singles=seg if T == 1 else seg[:0])
        xi, xo = _bf(n, inner + C)[:, inner:], _bf(n, inner)
        big = sv.ShortConv(w, torch.zeros(B, taps, C, dtype=bf, **dev), b)
        gw = _bf(inner)
        z, bias, table = torch.randn(n, 64, **dev), _bf(64), _bf(32000, 1024)
        gx, tok = _bf(n, 256), torch.randint(0, 32000, (n,)).int().cuda()
        y, u = _bf(n, W), _bf(n, 14336)
        t = _time([
            _graphed(lambda: sv.residual_norm(x, sv.Pending(d), 1e-5, wn)),
            _graphed(lambda: sv.residual_norm(x, sv.Pending(d), 1e-5, wn,
                                              groups=8)),
            _graphed(lambda: sv.residual_norm(
                x, sv.Pending(d, w1=wn), 1e-5, wn, groups=8, conv=cw,
                batch=batch)),
            _graphed(lambda: sv.residual_norm(
                x, sv.Pending(d2, coef=coef), 1e-5, copy=True, dtype=bf)),
            _graphed(lambda: sv.gated_norm(xo, gw, None, 1024, 1e-5)),
            _graphed(lambda: sv.gated_norm(y, wn, d, 128, 1e-5)),
            _graphed(lambda: sv.moe_plan(
                z, bias, sv.Routing(6, True, 8, 4), 0)),
            _graphed(lambda: sv.moe_plan(z, bias, 6, 0)),
            _graphed(lambda: sv.gelu_rows_(gx, table, tok, 256)),
            _graphed(lambda: sv.gelu_tanh_(gx)),
            _graphed(lambda: sv.gelu_tanh_(u))])
        like = ("residual_norm", t[0], 0, 12 * n * W)
        _report("residual_norm (groups)", t[1], 0, 12 * n * W, like, rows=n)
        _report("residual_norm (output norm, groups, convolution)", t[2], 0,
                (16 if T > 1 else 12 + 10) * n * W, like, rows=n)
        _report("residual_norm (experts' sum)", t[3], 0,
                (10 + 2 * top) * n * W, like, rows=n)
        _report("gated_norm (no gate)", t[4], 0, 4 * n * inner,
                ("gated_norm", t[5], 0, 6 * n * W), rows=n)
        if T > 1:
            (us,) = _time([_graphed(lambda: sv.short_conv(
                xi, big, seg, batch.chunks, silu=True))])
            _report("short_conv", us, 0, 4 * n * C,
                    ("gelu_tanh", t[10], 0, 4 * n * 14336), rows=n, channels=C)
        io = 4 * n * 64 + 12 * n * 6
        _report("moe_plan (sigmoid, groups)", t[6], 0, io,
                ("moe_plan", t[7], 0, io), rows=n, experts=64, top=6)
        _report("gelu_rows", t[8], 0, 6 * n * 256,
                ("gelu_tanh", t[9], 0, 4 * n * 256), rows=n)


def bench_state_models():
    _engine_models("Sutuvik", "Nesilorn")


def _engine_models(*names):
    for size in ("bench", "bench-fine"):
        _side_by_side(size, names)
        torch.cuda.empty_cache()


def _side_by_side(size, names):
    """Models of the serving engine, each in its configuration ``size``."""
    from neuronx_distributed_amd import models as zoo
    from neuronx_distributed_amd.inference import (InferenceEngine, StepEntry,
                                                   single_process_groups)
    from neuronx_distributed_amd.models import build_model

    single_process_groups()
    torch.manual_seed(0)
    cfgs = {n: getattr(zoo, f"get_{n.lower()}_config")(f"{n.lower()}-{size}")
            for n in names}
    models = {n: build_model(n, c, torch.bfloat16, "cuda")
              for n, c in cfgs.items()}
    out = {f"{n.lower()}_b_params": round(
        sum(p.numel() for p in m.parameters()) / 1e9, 2)
        for n, m in models.items()}
    print(json.dumps({"size": size, **out,
                      "width": cfgs[names[0]].hidden_size,
                      "layers": len(cfgs[names[0]].layers),
                      "data": "random weights"}), flush=True)

    def turns(fns, reps):
        best = [math.inf] * len(fns)
        for _ in range(reps):
            for i, f in enumerate(fns):
                torch.cuda.synchronize()
                t0 = time.perf_counter()
                f()
                torch.cuda.synchronize()
                best[i] = min(best[i], time.perf_counter() - t0)
        return best

    for B, T in ((1, 2048), (1, 4096), (4, 4096)):
        rows = torch.randint(0, 32000, (B, T)).tolist()

        def run(eng):
            eng.step([StepEntry(b, rows[b], [T - 1]) for b in range(B)])
            for b in range(B):
                eng.finish(b)

        engs = [InferenceEngine(m, max_tokens=B * T, max_seqs=B)
                for m in models.values()]
        best = turns([lambda e=e: run(e) for e in engs], 4)
        print(json.dumps({"prefill": {"batch": B, "tokens": T},
                          **{f"{n.lower()}_tokens_per_s": round(B * T / s)
                             for n, s in zip(models, best)}}), flush=True)
        del engs
        torch.cuda.empty_cache()
    for B, ctx in ((1, 2048), (32, 2048), (128, 2048)):
        steps = 8
        rows = torch.randint(0, 32000, (B, ctx)).tolist()
        engs = [InferenceEngine(m, max_tokens=B * (ctx + 64), max_seqs=B,
                                max_context=ctx + 64)
                for m in models.values()]
        for eng in engs:
            for b in range(B):
                eng.step([StepEntry(b, rows[b])])

        def decode(eng):
            tok = [1] * B
            for _ in range(steps):
                tok = eng.step([StepEntry(b, [tok[b]], [0]) for b in
                                range(B)]).argmax(-1).tolist()

        best = turns([lambda e=e: decode(e) for e in engs], 4)
        print(json.dumps({
            "decode": {"batch": B, "context": ctx},
            **{f"{n.lower()}_ms": round(s / steps * 1e3, 3)
               for n, s in zip(models, best)},
            **{f"{n.lower()}_tokens_per_s": round(B * steps / s)
               for n, s in zip(models, best)}}), flush=True)
        del engs
        torch.cuda.empty_cache()


# ---------------------------------------------------------------------------
# Pokepel beside Nesilorn and Voletar
# ---------------------------------------------------------------------------

def bench_retention_kernels():
    from dataclasses import replace

    from neuronx_distributed_amd import ops
    from neuronx_distributed_amd.ops import serving as sv

    dev = dict(device="cuda")
    # -- retention beside the decayed memory, each with its norm and gate ------
    H, D, E, eps = 32, 128, 128, 1e-5
    lgate = sv.decay_gate([0.99] * H, "cuda")
    gate = sv.TurnGate(lgate.decay, lgate.log2_decay, D ** -0.5,
                       sv.rotary_frequencies(1e4, D, "cuda"))
    w = _bf(H * E)
    for B, T in ((1, 4096), (4, 4096), (1, 1), (32, 1), (128, 1)):
        n = B * T
        q, k, v, g = _bf(n, 2 * H * (D + E)).split(
            (H * D, H * D, H * E, H * E), 1)
        S = torch.zeros(B, H, D, E, **dev)
        ctx = 64 if T == 1 else 0
        seg = _i32([(i, i * T, T, ctx) for i in range(B)])
        rows, first = sv.chunk_table(seg.tolist())
        tab = (_i32(rows), _i32(first)) if T > 1 else ()

        def like():
            o = sv.memory_mix(q, k, v, lgate, S, None, None, seg, H, *tab)
            return sv.gated_norm(o, w, g, H * E, eps)

        def mix():
            if T > 1:
                return sv.memory_mix(q, k, v, gate, S, None, None, seg, H,
                                     *tab, silu_gate=g, eps=eps)
            o = sv.memory_mix(q, k, v, gate, S, None, None, seg, H)
            return sv.gated_norm(o, None, g, E, eps, True, out=o)

        us, lus, mus, lmus = _time([
            _graphed(mix), _graphed(like),
            _graphed(lambda: sv.memory_mix(q, k, v, gate, S, None, None, seg,
                                           H, *tab)),
            _graphed(lambda: sv.memory_mix(q, k, v, lgate, S, None, None, seg,
                                           H, *tab))])
        cs = 64 if T > 1 else 1
        fl = 2 * n * H * (cs / 2 * (D + E) + 2 * D * E)
        io = 4 * n * H * (D + E) + (8 if ctx else 4) * B * H * D * E
        # every product of split operands at its MFMA cost
        f5 = 2 * n * H * (cs / 2 * (3 * D + 3 * E) + 10 * D * E)
        extra = {"roofline_32bit_us": round(
            max(f5 / PEAK_FLOPS, io / PEAK_BYTES) * 1e6, 2)} if T > 1 else {}
        kw = dict(batch=B, tokens=T, heads=H, dim=D, vdim=E, **extra)
        name = "chunks" if T > 1 else "steps"
        _report(f"retention_{name} (rotation)", mus, fl, io,
                ("decayed memory", lmus, fl, io), **kw)
        _report(f"retention_{name} (rotation, norm, gate)", us, fl,
                io + 2 * n * H * E, ("decayed memory, gated_norm", lus, fl,
                                     io + 2 * n * H * E), **kw)
    # -- latent attention with a sink and neighbouring pairs --------------------
    H, D, P, E, R = 32, 128, 64, 128, 512
    scale = (D + P) ** -0.5
    sink = _bf(H)
    for B, T, ctx in ((1, 4096, 0), (1, 8192, 0), (1, 1, 4096),
                      (32, 1, 1024), (32, 1, 4096), (128, 1, 4096)):
        b, lw, cache, q, kv, g = _latent_case(sv, B, T, ctx, H, D, P, E, R)
        w = replace(lw, amplitude=1.14, pairs=True, sink=sink)
        if T > 1:
            pages, table = sv.key_spans([(0, 0, T, 0)],
                                        b.block_table.tolist(), 0)
            b.spans = {0: sv.KeySpans(_i32(pages), _i32(table))}
        fns = [_graphed(lambda x=x: sv.latent_attention(
            q, kv, g, b, cache, x, H, D, E, scale, 1e-5)) for x in (w, lw)]
        pairs = B * sum(ctx + i + 1 for i in range(T))
        if T > 1:
            kve, ws = _bf(T, H * (D + E)), _bf(T, R + P)
            out = torch.empty(T, H * E, dtype=torch.bfloat16, **dev)
            fns += [_graphed(lambda s=s: sv.expanded_attention(
                q, g, kve, ws, b.tiles, b.spans[0], H, D, E, scale, 0, out,
                s)) for s in (sink, None)]
            fl = 2 * pairs * H * (D + P + E)
            io = 2 * T * (H * (D + P + 2 * E) + R + P) + \
                2 * T * H * (D + E)
            all_fl, all_io = fl + 2 * T * R * H * (D + E), io
        else:
            ql = _bf(B, H * (R + P))
            fns += [_graphed(lambda s=s: sv.latent_rows(
                ql, cache, R, b.pos, b.seq, b.block_table, H, scale, 0,
                ctx + 1, s)) for s in (sink, None)]
            fl = 2 * pairs * H * (2 * R + P)
            io = 2 * B * (ctx + 1) * (R + P) + 2 * B * H * (2 * R + P)
            all_fl = fl + 2 * B * H * R * (D + E)
            all_io = io + 2 * H * (D + E) * R + 2 * B * H * (D + P + 2 * E)
        t = _time(fns)
        kw = dict(batch=B, tokens=T, context=ctx)
        _report("latent_attention (sink, pairs)", t[0], all_fl, all_io,
                ("latent_attention", t[1], all_fl, all_io), **kw)
        name = "attn_tiles on expanded keys" if T > 1 else "latent_rows"
        _report(name + " (sink)", t[2], fl, io, (name, t[3], fl, io), **kw)
    # -- residual, activations, routing -----------------------------------------
    for T in (32, 4096):
        Wd, F, top = 4096, 14336, 2
        x, d, d1, plus, wn = (torch.randn(T, Wd, **dev), _bf(T, Wd),
                              _bf(T, Wd), _bf(T, Wd), _bf(Wd))
        d2, coef = _bf(T * top, Wd), torch.rand(T, top, **dev)
        gates = _bf(T, 2 * Wd)
        A = sv.Branch(d1, gate=gates[:, :Wd], bias=wn)
        dense = sv.Branch(plus, gate=gates[:, Wd:], bias=wn)
        moe = sv.Branch(d2, coef, plus, gates[:, Wd:], wn)
        u, gu, act = _bf(T, F + 64), _bf(T, 2 * F), _bf(4)
        z = torch.randn(T, 64, **dev)
        t = _time([
            _graphed(lambda: sv.residual_norm(
                x, sv.Pending(branches=[A, dense]), 1e-6, wn)),
            _graphed(lambda: sv.residual_norm(
                x, sv.Pending(branches=[A, moe]), 1e-6, wn)),
            _graphed(lambda: sv.residual_norm(
                x, sv.Pending(d, d1, wn, wn, 0.5), 1e-6, wn)),
            _graphed(lambda: sv.poly_norm(u[:, :F], act, 1e-6)),
            _graphed(lambda: sv.silu_mul(gu)),
            _graphed(lambda: ops.swiglu(gu)),
            _graphed(lambda: sv.gelu_tanh_(u)),
            _graphed(lambda: sv.moe_plan(z, None, sv.Routing(
                6, groups=8, keep=4, softmax=True, best=1), 0)),
            _graphed(lambda: sv.moe_plan(z, None, 6, 0)),
            _graphed(lambda: sv.gated_norm(d, None, d1, 128, 1e-5, True)),
            _graphed(lambda: sv.gated_norm(d, wn, d1, 128, 1e-5))])
        n = T * Wd
        like = ("residual_norm (two branches)", t[2], 0, 14 * n)
        _report("residual_norm (gated branches)", t[0], 0, 18 * n, like,
                rows=T)
        _report("residual_norm (gated branches, experts and a shared one)",
                t[1], 0, (18 + 2 * top) * n, like, rows=T)
        _report("poly_norm", t[3], 0, 4 * T * F,
                ("gelu_tanh", t[6], 0, 4 * T * F), rows=T)
        _report("silu_mul", t[4], 0, 6 * T * F,
                ("swiglu", t[5], 0, 6 * T * F), rows=T)
        io = 4 * T * 64 + 12 * T * 6
        _report("moe_plan (softmax, groups)", t[7], 0, io,
                ("moe_plan", t[8], 0, io), rows=T, experts=64, top=6)
        _report("gated_norm (silu, no weight)", t[9], 0, 6 * n,
                ("gated_norm", t[10], 0, 6 * n), rows=T)


def bench_retention_models():
    _engine_models("Pokepel", "Nesilorn")


DESIGNS = {"voletar": (bench_kernels, bench_models),
           "nesilorn": (bench_latent_kernels, bench_latent_models),
           "sutuvik": (bench_state_kernels, bench_state_models),
           "pokepel": (bench_retention_kernels, bench_retention_models)}


def main(what="all", design="all"):
    torch.cuda.set_device(0)
    for name, (kernels, models) in DESIGNS.items():
        if design in ("all", name):
            if what in ("all", "kernels"):
                kernels()
            if what in ("all", "models"):
                models()


if __name__ == "__main__":
    import sys

    main(*sys.argv[1:3])
