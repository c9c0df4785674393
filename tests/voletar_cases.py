"""Small Voletar configurations and weights for the tests."""

import torch


def lightning(heads, dim, vdim, decay, ff=None):
    return {"type": "lightning", "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "decay": decay},
        "mlp": ff and {"kind": "dense", "ff": ff}}


def parallel(left, right, ff=None):
    H, G, D, E, size, keep, scale = left
    h, d, e, cap = right
    return {"type": "parallel", "mixer": {
        "left": {"heads": H, "kv_heads": G, "dim": D, "vdim": E,
                 "scale": scale, "mask": {"size": size, "keep_first": keep}},
        "right": {"heads": h, "dim": d, "vdim": e, "gate_cap": cap}},
        "mlp": ff and {"kind": "dense", "ff": ff}}


def config(vocab, width, layers, loop, eps=1e-5, cap=25.0):
    return {"architecture": "Voletar", "vocab": vocab, "width": width,
            "layers": layers, "loop": loop, "norm": {"eps": eps},
            "logit_softcap": cap}


CASES = {
    # grouped heads, unequal sizes, a loop in the middle, mlps everywhere
    "middle_loop": config(210, 96, [
        parallel((6, 2, 40, 24, 70, 5, 0.3), (2, 32, 48, 4.0), 112),
        lightning(3, 24, 40, [0.2, 0.95, 0.9995], 64),
        parallel((4, 1, 16, 32, 33, 0, 0.5), (3, 16, 8, 9.0)),
        lightning(2, 72, 16, [1.0, 0.0]),
        parallel((2, 2, 64, 72, 130, 70, 0.2), (1, 80, 104, 15.0), 80),
    ], {"start": 1, "stop": 4, "times": 3}),
    # sizes that are no multiple of 8 or of 4
    "odd": config(77, 50, [
        lightning(3, 10, 7, [0.5, 0.9, 0.99], 33),
        parallel((3, 1, 20, 12, 18, 3, 0.4), (2, 9, 21, 6.0), 30),
    ], {"start": 0, "stop": 2, "times": 2}, eps=1e-3, cap=5.0),
    # several layers of a kind in a row, every window another, looped once
    "rows": config(128, 128, [
        lightning(1, 128, 128, [0.97]),
        lightning(4, 32, 64, [0.7, 0.8, 0.9, 0.999], 96),
        parallel((8, 2, 32, 32, 64, 64, 0.25), (2, 64, 32, 15.0)),
        parallel((2, 1, 128, 96, 100, 1, 0.125), (1, 128, 64, 30.0), 64),
    ], {"start": 2, "stop": 4, "times": 1}),
    # no loop; no attention at all, so no pages either
    "memory_only": config(96, 64, [
        lightning(2, 32, 32, [0.9, 0.98], 64),
        lightning(2, 16, 64, [0.99, 0.3]),
    ], None),
}


def tensors(cfg):
    """(name, shape) of every tensor of a configuration."""
    W, V = cfg["width"], cfg["vocab"]
    out = [("embed", (V, W)), ("final.norm", (W,)), ("head", (V, W))]
    if cfg["loop"]:
        out += [("loop.in", (W, 2 * W)),
                ("loop.step", (cfg["loop"]["times"], W))]
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        out.append((p + "norm1", (W,)))
        if L["type"] == "lightning":
            qk, v = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            out += [(p + "mix." + n, s) for n, s in (
                ("q", (qk, W)), ("k", (qk, W)), ("v", (v, W)), ("g", (v, W)),
                ("o", (W, v)), ("norm", (v,)))]
        else:
            l, r = m["left"], m["right"]
            out += [(p + "mix.left." + n, s) for n, s in (
                ("q", (l["heads"] * l["dim"], W)),
                ("k", (l["kv_heads"] * l["dim"], W)),
                ("v", (l["kv_heads"] * l["vdim"], W)),
                ("o", (W, l["heads"] * l["vdim"])), ("out", (W,)))]
            qk, v = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            out += [(p + "mix.right." + n, s) for n, s in (
                ("q", (qk, W)), ("k", (qk, W)), ("v", (v, W)), ("g", (v, W)),
                ("o", (W, v)), ("norm", (v,)), ("i", (r["heads"], W)),
                ("i.b", (r["heads"],)), ("f", (r["heads"], W)),
                ("f.b", (r["heads"],)), ("out", (W,)))]
        if L["mlp"]:
            ff = L["mlp"]["ff"]
            out += [(p + "norm2", (W,)), (p + "mlp.up", (ff, W)),
                    (p + "mlp.down", (W, ff))]
    return out


def weights(cfg, seed=0):
    """Random bf16 weights under which every part of the model shows:
    peaked attention, forget gates near one, lively input gates."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensors(cfg):
        t = torch.randn(*shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if name.endswith(".f.b"):
            t = 3.0 + t
        elif name.endswith(".i.b"):
            t = 0.5 * t
        elif len(shape) == 1:                       # norm weights
            t = 1.0 + 0.2 * t
        elif name == "loop.step" or name == "embed":
            pass
        else:
            t = t * shape[1] ** -0.5
            if last == "head":
                t = 3.0 * t
            if last in ("q", "k") and ".left." in name:
                t = 1.6 * t
        out[name] = t.to(torch.bfloat16)
    return out


def save(cfg, w, folder):
    import json

    from safetensors.torch import save_file

    with open(folder / "config.json", "w") as f:
        json.dump(cfg, f)
    save_file(w, str(folder / "model.safetensors"))
