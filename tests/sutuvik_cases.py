"""Small Sutuvik configurations and weights for the tests."""

import math

import torch


def mamba2(heads, vdim, state, groups=1, conv=4, norm_groups=1):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state,
                      "groups": groups, "conv": conv,
                      "norm_groups": norm_groups}


def attention(heads, kv_heads, dim, vdim, scale, v_mix=True, coef=0.4,
              every=50):
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                         "vdim": vdim, "scale": scale, "v_mix": v_mix,
                         "q_temp": {"coef": coef, "every": every}}


def attention_2(heads, kv_heads, dim, vdim, scale, softcap, dims, base=1e4,
                v_mix=True, scaling=(4.0, 1.0, 4.0, 128)):
    sc = dict(zip(("factor", "low", "high", "original"), scaling)) \
        if scaling else None
    return "attention_2", {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "scale": scale, "softcap": softcap, "v_mix": v_mix,
        "rot": {"base": base, "dims": dims, "scaling": sc}}


def moe(ff, experts, top, count, keep):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {
        "experts": experts, "top": top,
        "groups": {"count": count, "keep": keep}}}


def config(vocab, width, layers, groups, taps=4, side=16, eps=1e-5,
           scale=0.6):
    return {"architecture": "Sutuvik", "vocab": vocab, "width": width,
            "norm": {"eps": eps, "groups": groups}, "canon": {"taps": taps},
            "token_side": {"dim": side}, "logit_scale": scale,
            "layers": [{"type": m[0], "mixer": m[1], "mlp": f}
                       for m, f in layers]}


CASES = {
    # every size another; heads share keys in groups everywhere
    "mixed": config(210, 96, [
        (mamba2(6, 40, 24, 3, 3, 2), moe(40, 8, 2, 4, 2)),
        (attention(6, 2, 16, 24, 0.3), None),
        (attention_2(4, 1, 72, 48, 0.12, 9.0, 40), moe(72, 6, 3, 2, 1)),
        (mamba2(4, 72, 80, 2, 4, 1), None),
        (attention_2(8, 2, 32, 24, 0.2, 4.0, 32, 77.0), moe(24, 9, 4, 3, 3)),
        (attention(3, 1, 40, 48, 0.2, True, 1.5, 7), moe(40, 4, 1, 2, 1)),
    ], groups=3, taps=3),
    # sizes that are no multiple of 8 or of 4; long and short filters
    "odd": config(77, 50, [
        (attention_2(3, 1, 11, 10, 0.5, 3.0, 6, 9.0), moe(27, 6, 2, 3, 2)),
        (mamba2(3, 7, 13, 1, 5, 3), moe(33, 4, 3, 1, 1)),
        (attention(2, 2, 9, 5, 0.5, True, 0.7, 3), moe(30, 7, 1, 7, 3)),
        (mamba2(2, 33, 5, 2, 2, 1), None),
    ], groups=5, taps=7, side=9, eps=1e-3, scale=1.7),
    # states of several tiles, values that are not mixed, one norm group, filters
    # of two taps
    "wide": config(128, 128, [
        (mamba2(4, 96, 136, 1, 4, 4), moe(64, 8, 4, 4, 3)),
        (attention(4, 4, 144, 64, 0.15, False), moe(48, 8, 3, 2, 1)),
        (attention_2(2, 2, 64, 160, 0.3, 20.0, 16, 1e6, False, None),
         moe(32, 6, 2, 3, 2)),
        (mamba2(2, 16, 300, 2, 4, 2), None),
    ], groups=1, taps=2, side=32, scale=1.0),
    # nothing is paged
    "memories": config(90, 64, [
        (mamba2(4, 32, 32, 4, 4, 4), moe(32, 6, 2, 2, 1)),
        (mamba2(2, 24, 16, 1, 1, 1), moe(40, 5, 5, 1, 1)),
    ], groups=2, taps=1, side=8),
}


def tensors(cfg):
    """(name, shape) of every tensor of a configuration."""
    W, V, L = cfg["width"], cfg["vocab"], cfg["layers"]
    dim = cfg["token_side"]["dim"]
    out = [("embed", (V, W)), ("embed.norm", (W,)),
           ("side.embed", (V, len(L) * dim)), ("final.norm", (W,))]
    for i, layer in enumerate(L):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        H = m["heads"]
        out += [(p + "norm1", (W,)), (p + "canon1", (W, cfg["canon"]["taps"])),
                (p + "side.gate", (dim, W)), (p + "side.proj", (W, dim)),
                (p + "side.norm", (W,))]
        if layer["type"] == "mamba2":
            inner, gn = H * m["vdim"], m["groups"] * m["state"]
            c = inner + 2 * gn
            mix = [("in", (inner + c + H, W)), ("conv", (c, m["conv"])),
                   ("conv.b", (c,)), ("dt_bias", (H,)), ("A_log", (H,)),
                   ("D", (H,)), ("norm", (inner,)), ("o", (W, inner))]
        else:
            G, D, E = m["kv_heads"], m["dim"], m["vdim"]
            mix = [("q", (H * D, W)), ("k", (G * D, W)), ("v", (G * E, W)),
                   ("o", (W, H * E))]
            if m["v_mix"]:
                mix.append(("vmix", ()))
            if layer["type"] == "attention":
                mix += [("q.norm", (D,)), ("k.norm", (D,)), ("sink", (H,)),
                        ("g", (H, W))]
            else:
                mix.append(("temp", (H,)))
        out += [(p + "mix." + n, s) for n, s in mix]
        if f is None:
            continue
        n, ff = f["router"]["experts"], f["expert"]["ff"]
        out += [(p + "norm2", (W,)), (p + "mlp.router", (n, W)),
                (p + "mlp.correction", (n,))]
        for e in range(n):
            out += [(f"{p}mlp.e{e}.gate", (ff, W)),
                    (f"{p}mlp.e{e}.up", (ff, W)),
                    (f"{p}mlp.e{e}.down", (W, ff))]
    return out


def weights(cfg, seed=0):
    """Random bf16 weights under which every part of the model shows: peaked
    attention, sinks that take a good part, decays from one to many tokens,
    corrections that change choices.  The first columns of the embedding hold
    each token's liking of the experts; nothing else writes them and only the
    routers read them, so that rounding decides (nearly) no choice."""
    g = torch.Generator().manual_seed(seed)
    n = max([L["mlp"]["router"]["experts"] for L in cfg["layers"]
             if L["mlp"]], default=0)
    n = min(n, cfg["width"] // 4)
    out = {}
    for name, shape in tensors(cfg):
        t = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last in ("norm", "norm1", "norm2"):
            t = 1.0 + 0.2 * t
            if name in ("final.norm",) or last == "norm1" or "side" in name:
                t[:n] = 0.0
        elif last == "embed" and name == "embed":
            t[:, :n] = torch.stack([torch.randperm(n, generator=g)
                                    for _ in range(shape[0])]).float()
            t[:, :n] = 3.0 * (t[:, :n] + 0.5) / n - 1.5
        elif last == "router":
            t = 0.01 * t
            t[:, :n] = 2.0 * torch.eye(n)[torch.randint(
                0, n, (shape[0],), generator=g)]
            perm = torch.randperm(n, generator=g)
            m = min(n, shape[0])
            t[:m, :n] = 2.0 * torch.eye(n)[perm[:m]]
        elif last == "correction":
            t = 0.3 * t - 0.2
        elif last in ("sink", "D"):
            t = 0.5 + t
        elif last == "temp":
            t = 2.0 + t
        elif last == "vmix":
            t = 0.5 + 0.1 * t
        elif last == "dt_bias":
            t = t - 2.0
        elif last == "A_log":
            t = t.clamp(-2.0, 2.0)
        elif name.endswith("conv.b"):
            t = 0.2 * t
        elif last in ("canon1", "conv"):
            t = t * shape[1] ** -0.5
        else:
            t = t * (shape[1] if len(shape) > 1 else 1) ** -0.5
            if last in ("o", "down"):
                t[:n] = 0.0
        out[name] = t.to(torch.bfloat16)
    return out


_steady = {}


def steady_tokens(case):
    """The third of a case's vocabulary for which the routers' choices are
    least close, so that rounding decides none of them."""
    import sutuvik_oracle as so

    if case not in _steady:
        cfg, w = CASES[case], weights(CASES[case])
        gap = []
        for t in range(cfg["vocab"]):
            m = []
            so.forward(cfg, w, [t], margins=m)
            gap.append(min(x.item() for x in m))
        order = sorted(range(cfg["vocab"]), key=lambda t: -gap[t])
        _steady[case] = sorted(order[:cfg["vocab"] // 3])
    return _steady[case]


_prompts = {}


def prompt(case, n, seed=0):
    """Random steady tokens; of some draws, the first that leaves no choice
    close in its own context either (or the best)."""
    import sutuvik_oracle as so

    if (case, n, seed) not in _prompts:
        cfg, some = CASES[case], steady_tokens(case)
        w = weights(cfg)
        best, toks = -1.0, None
        for draw in range(12):
            g = torch.Generator().manual_seed(1000 * draw + seed)
            t = [some[i] for i in torch.randint(0, len(some), (n,),
                                                generator=g)]
            m = []
            so.forward(cfg, w, t, torch.float32, margins=m)
            gap = min(x.min().item() for x in m)
            if gap > best:
                best, toks = gap, t
            if best > 0.006:
                break
        _prompts[case, n, seed] = toks
    return _prompts[case, n, seed]


def save(cfg, w, folder):
    import json

    from safetensors.torch import save_file

    with open(folder / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file(w, str(folder / "model.safetensors"))


def attention_case(T, H, G, D, E, seed, far):
    """Queries, keys and values (float64, heads apart) in which the keys at
    ``far`` stand out for every query: a fault at one of them shows."""
    g = torch.Generator().manual_seed(seed)
    q, k, v = (torch.randn(T, n, d, generator=g, dtype=torch.float64)
               for n, d in ((H, D), (G, D), (G, E)))
    q[..., 0] = math.sqrt(D)
    for i, j in enumerate(far):
        k[j, :, 0] = math.sqrt(D) * (1.0 + 0.05 * i)
    return q, k, v
