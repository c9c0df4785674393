"""Small Pokepel configurations and weights for the tests."""

import json
import math

import torch


def latent(heads, dim, rot, vdim, rank, scale, base=1e4,
           scaling=(3.0, 40, 2.5, 0.6)):
    sc = dict(zip(("factor", "original", "fast", "slow"), scaling)) \
        if scaling else None
    return "latent_attention", {
        "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
        "kv_rank": rank, "scale": scale,
        "rot": {"base": base, "dims": rot, "scaling": sc}}


def retention(heads, dim, vdim, dims, decay, base=1e4):
    assert len(decay) == heads
    return "retention", {"heads": heads, "dim": dim, "vdim": vdim,
                         "decay": decay, "rot": {"base": base, "dims": dims}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, count, keep, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared},
            "router": {"experts": experts, "top": top,
                       "groups": {"count": count, "keep": keep}}}


def config(vocab, width, layers, eps=1e-5):
    return {"architecture": "Pokepel", "vocab": vocab, "width": width,
            "norm": {"eps": eps},
            "layers": [{"type": m[0], "mixer": m[1], "mlp": f}
                       for m, f in layers]}


CASES = {
    # every size another, all kinds of layers
    "mixed": config(210, 96, [
        (retention(3, 40, 24, 32, [0.9, 0.99, 0.999]),
         moe(40, 8, 2, 4, 2, 56)),
        (latent(6, 24, 16, 40, 48, 0.3), dense(112)),
        (latent(3, 16, 32, 24, 72, 0.25, 500.0, (8.0, 300, 6.0, 1.0)),
         moe(72, 6, 3, 2, 1, 24)),
        (retention(4, 72, 48, 72, [0.5, 0.97, 1.0, 0.995], 77.0), None),
        (latent(5, 40, 8, 16, 40, 0.3, 50.0), moe(24, 9, 4, 3, 3, 136)),
        (retention(2, 24, 136, 8, [0.98, 0.9995]), dense(64)),
    ]),
    # sizes that are no multiple of 8 or of 4; one group, one expert a group
    "odd": config(77, 50, [
        (latent(3, 10, 6, 7, 21, 0.5, 9.0), moe(27, 6, 2, 3, 2, 13)),
        (retention(3, 13, 7, 6, [0.8, 0.95, 0.99], 300.0), dense(33)),
        (latent(1, 9, 2, 12, 13, 0.6), moe(33, 4, 3, 1, 1, 50)),
        (retention(1, 6, 33, 6, [0.97]), moe(30, 7, 1, 7, 3, 9)),
        (latent(2, 7, 10, 5, 30, 0.4, 77.0), None),
    ], eps=1e-3),
    # more than 32 heads, states and latents of several tiles, rotations that
    # are not scaled
    "wide": config(128, 128, [
        (latent(36, 8, 8, 16, 256, 0.9, 1e4, None), moe(64, 4, 4, 1, 1, 64)),
        (retention(2, 136, 160, 128, [0.99, 0.96]), dense(256)),
        (latent(2, 128, 64, 128, 320, 0.12, 1e5), moe(48, 8, 3, 4, 3, 128)),
        (retention(2, 200, 64, 24, [0.99, 0.96]), moe(32, 8, 2, 2, 1, 32)),
    ]),
    # nothing is paged
    "memories": config(90, 64, [
        (retention(4, 32, 32, 32, [0.9, 0.95, 0.99, 0.999]),
         moe(32, 6, 2, 2, 1, 40)),
        (retention(2, 16, 24, 8, [0.97, 0.9999]), dense(40)),
    ]),
}


def tensors(cfg):
    """(name, shape) of every tensor of a configuration."""
    W, V = cfg["width"], cfg["vocab"]
    out = [("embed", (V, W)), ("final.norm", (W,)), ("head", (V, W))]
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", layer["mixer"], layer["mlp"]
        H, D, E = m["heads"], m["dim"], m["vdim"]
        out += [(p + "norm1", (W,)), (p + "rg1", (W, W)), (p + "rg1.b", (W,))]
        if layer["type"] == "retention":
            mix = [("q", (H * D, W)), ("k", (H * D, W))]
            mix += [("v", (H * E, W))]
        else:
            P, R = m["rot_dim"], m["kv_rank"]
            mix = [("q", (H * (D + P), W)), ("dkv", (R + P, W)),
                   ("dkv.norm", (R,)), ("uk", (H * D, R)),
                   ("uv", (H * E, R)), ("sink", (H,))]
        mix += [("g", (H * E, W)), ("o", (W, H * E))]
        out += [(p + "mix." + n, s) for n, s in mix]
        if f is None:
            continue
        out += [(p + "rg2", (W, W)), (p + "rg2.b", (W,))]
        p += "mlp."
        if f["kind"] == "dense":
            out += [(p + "up", (f["ff"], W)), (p + "down", (W, f["ff"])),
                    (p + "act", (4,))]
            continue
        n = f["router"]["experts"]
        out.append((p + "router", (n, W)))
        for e, ff in [(f"e{e}", f["expert"]["ff"]) for e in range(n)] + \
                [("shared", f["shared"]["ff"])]:
            out += [(f"{p}{e}.gate", (ff, W)), (f"{p}{e}.up", (ff, W)),
                    (f"{p}{e}.down", (W, ff))]
    return out


def weights(cfg, seed=0):
    """Random bf16 weights under which every part of the model shows: peaked
    attention, sinks that take a good part, gates on both sides.  The first
    columns of the embedding hold each token's liking of the experts; nothing
    else writes them and only the routers read them, so that rounding decides
    (nearly) no choice."""
    g = torch.Generator().manual_seed(seed)
    n = max([L["mlp"]["router"]["experts"] for L in cfg["layers"]
             if L["mlp"] and L["mlp"]["kind"] == "moe"], default=0)
    out = {}
    for name, shape in tensors(cfg):
        t = torch.randn(shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last in ("norm", "norm1"):
            t = 1.0 + 0.2 * t
            if last == "norm1":
                t[:n] = 1.0
        elif last == "embed":
            t[:, :n] = torch.stack([torch.randperm(n, generator=g)
                                    for _ in range(shape[0])]).float()
            t[:, :n] = 3.0 * (t[:, :n] + 0.5) / max(n, 1) - 1.5
        elif last == "router":
            t = 0.01 * t
            perm = torch.randperm(n, generator=g)[:shape[0]]
            t[:, :n] = 2.0 * torch.eye(n)[perm]
        elif last == "sink":
            t = 1.0 + t
        elif last == "act":
            t = torch.tensor([0.7, -0.5, 0.9, 0.3]) + 0.1 * t
        elif last == "b":
            t = 0.5 * t
        else:
            t = t * shape[1] ** -0.5
            if last in ("o", "down"):
                t[:n] = 0.0
            else:             # only the routers read those columns
                t[..., :n] = 0.0 if shape[1] == cfg["width"] else \
                    t[..., :n]
        out[name] = t.to(torch.bfloat16)
    return out


_prompts = {}


def prompt(case, n, seed=0):
    """Random tokens; of some draws, the first that leaves no router's choice
    close (or the best)."""
    import pokepel_oracle as po

    if (case, n, seed) not in _prompts:
        cfg, w = CASES[case], weights(CASES[case])
        best, toks = -1.0, None
        for draw in range(8):
            g = torch.Generator().manual_seed(1000 * draw + seed)
            t = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
            m = []
            po.forward(cfg, w, t, torch.float32, margins=m)
            gap = min(x.min().item() for x in m) if m else math.inf
            if gap > best:
                best, toks = gap, t
            if best > 0.1:
                break
        _prompts[case, n, seed] = toks
    return _prompts[case, n, seed]


def save(cfg, w, folder):
    from safetensors.torch import save_file

    with open(folder / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file(w, str(folder / "model.safetensors"))
