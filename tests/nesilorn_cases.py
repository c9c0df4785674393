"""Small Nesilorn configurations and weights for the tests."""

import torch


def mixer(heads, dim, rot, vdim, rank, window, scale, base=1e4):
    return {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
            "kv_rank": rank, "scale": scale, "rot": {"base": base,
                                                     "dims": rot},
            "mask": {"size": window} if window else None}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, limit):
    return {"kind": "moe", "router": {"experts": experts, "top": top},
            "expert": {"ff": ff, "limit": limit}}


def config(vocab, width, layers, eps=1e-5, scale=2.5):
    return {"architecture": "Nesilorn", "vocab": vocab, "width": width,
            "embedding": {"scale": scale}, "norm": {"eps": eps},
            "layers": [{"type": "latent_attention", "mixer": m, "mlp": f}
                       for m, f in layers]}


CASES = {
    # every size and window another, all kinds of feed-forward
    "mixed": config(230, 96, [
        (mixer(3, 24, 16, 40, 48, 70, 0.17), moe(72, 5, 2, 0.9)),
        (mixer(5, 40, 8, 16, 72, 33, 0.15, 500.0), dense(112)),
        (mixer(2, 16, 32, 64, 128, 130, 0.13, 1e6), None),
        (mixer(4, 32, 24, 24, 40, 64, 0.14), moe(40, 9, 4, 2.0)),
    ]),
    # sizes that are no multiple of 8 or of 4; one expert chosen
    "odd": config(77, 50, [
        (mixer(3, 10, 6, 7, 21, 18, 0.35), moe(27, 3, 1, 0.6)),
        (mixer(1, 9, 2, 12, 13, 65, 0.4, 77.0), moe(33, 4, 3, 1.1)),
        (mixer(2, 7, 10, 5, 30, 3, 0.25), dense(30)),
    ], eps=1e-3, scale=0.7),
    # more than 32 heads, more latents than keys, all experts chosen
    "heads": config(128, 128, [
        (mixer(36, 8, 8, 16, 256, 100, 0.9), moe(64, 4, 4, 1.5)),
        (mixer(40, 16, 64, 8, 320, 65, 0.4), moe(48, 16, 5, 3.0)),
    ], scale=1.0),
    # no window: everything stays visible
    "causal": config(90, 64, [
        (mixer(2, 32, 16, 32, 64, None, 0.4), moe(32, 6, 2, 1.0)),
        (mixer(2, 16, 16, 16, 32, None, 0.5), dense(64)),
    ]),
}


def tensors(cfg):
    """(name, shape) of every tensor of a configuration."""
    W, V = cfg["width"], cfg["vocab"]
    out = [("embed", (V, W)), ("final.norm", (W,))]
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L["mlp"]
        H, D, P = m["heads"], m["dim"], m["rot_dim"]
        E, R = m["vdim"], m["kv_rank"]
        out += [(p + "norm1", (W,))] + [(p + "mix." + n, s) for n, s in (
            ("q", (H * (D + P), W)), ("dkv", (R + P, W)), ("dkv.norm", (R,)),
            ("uk", (H * D, R)), ("uv", (H * E, R)), ("g", (H * E, W)),
            ("o", (W, H * E)))]
        if f is None:
            continue
        out.append((p + "norm2", (W,)))
        if f["kind"] == "dense":
            out += [(p + "mlp.up", (f["ff"], W)),
                    (p + "mlp.down", (W, f["ff"]))]
            continue
        n, ff = f["router"]["experts"], f["expert"]["ff"]
        out += [(p + "mlp.router", (n, W)), (p + "mlp.router.b", (n,))]
        for e in range(n):
            out += [(f"{p}mlp.e{e}.gate", (ff, W)),
                    (f"{p}mlp.e{e}.up", (ff, W)),
                    (f"{p}mlp.e{e}.down", (W, ff))]
    return out


def weights(cfg, seed=0):
    """Random bf16 weights under which every part of the model shows: peaked
    attention, activations on both sides of the experts' limits.  The first
    columns of the embedding hold each token's ranking of the experts; the
    norms keep the layers and the logits off them and the routers read little
    else, so that rounding decides no choice."""
    g = torch.Generator().manual_seed(seed)
    n = max([L["mlp"]["router"]["experts"] for L in cfg["layers"]
             if L["mlp"] and L["mlp"]["kind"] == "moe"], default=0)
    out = {}
    for name, shape in tensors(cfg):
        t = torch.randn(*shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if name.endswith("router.b"):
            t = 0.1 * t
        elif name.endswith("dkv.norm"):
            t = 1.0 + 0.2 * t
        elif len(shape) == 1:               # norms, stored around zero
            t = 0.2 * t
            t[:n] = -1.0
        elif last == "embed":
            rank = torch.stack([torch.randperm(n, generator=g)
                                for _ in range(shape[0])]).float()
            t[:, :n] = 0.25 * (rank - (n - 1) / 2)
            t = t / cfg["embedding"]["scale"]
        elif last == "router":
            t = 0.01 * t
            t[:, :n] = 4.0 * torch.eye(n)[torch.randperm(
                n, generator=g)[:shape[0]]]
        else:
            t = t * shape[1] ** -0.5
        out[name] = t.to(torch.bfloat16)
    return out


def save(cfg, w, folder):
    import json

    from safetensors.torch import save_file

    with open(folder / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file(w, str(folder / "model.safetensors"))
