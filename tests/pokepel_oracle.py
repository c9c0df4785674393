"""Plain, slow implementation of the Pokepel design for the tests.

One function per mechanism, every weight used as it is stored, the recurrence
one token after another.  It shares no code with the package: sizes come from
the config dictionary, weights from a name -> tensor dictionary.  ``dtype`` is
the arithmetic (float64 for a golden answer, float32 to see rounding).
"""

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm(x, weight, eps):
    return rms(x, eps) * weight


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def ramp(i, rot):
    """How far pair i is slowed by the scaling: 0 kept, 1 by the factor."""
    sc, n = rot["scaling"], rot["dims"]

    def pair_of(turns):
        return n * math.log(sc["original"] / (2 * math.pi * turns)) / \
            (2 * math.log(rot["base"]))

    lo = max(math.floor(pair_of(sc["fast"])), 0)
    hi = min(math.ceil(pair_of(sc["slow"])), n - 1)
    return min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)


def frequency(i, rot):
    """Radians a position of pair i."""
    f = rot["base"] ** (-2.0 * i / rot["dims"])
    if rot.get("scaling"):
        r = ramp(i, rot)
        f = f / rot["scaling"]["factor"] * r + f * (1.0 - r)
    return f


def amplitude(rot):
    """What cos and sin are multiplied by."""
    if not rot.get("scaling"):
        return 1.0
    return 0.1 * math.log(rot["scaling"]["factor"]) + 1.0


def _turn(x, positions, rot, first, second):
    """x (T, ..., n): elements first(i) and second(i) turn together."""
    out = x.clone()
    p = torch.as_tensor(list(positions), dtype=torch.float64)
    p = p.view(-1, *[1] * (x.dim() - 2))
    for i in range(rot["dims"] // 2):
        a = p * frequency(i, rot)
        c = (torch.cos(a) * amplitude(rot)).to(x.dtype)
        s = (torch.sin(a) * amplitude(rot)).to(x.dtype)
        u, v = x[..., first(i)], x[..., second(i)]
        out[..., first(i)] = u * c - v * s
        out[..., second(i)] = v * c + u * s
    return out


def rotate_pairs(x, positions, rot):
    """Neighbours turn together."""
    return _turn(x, positions, rot, lambda i: 2 * i, lambda i: 2 * i + 1)


def rotate_halves(x, positions, rot):
    """The first and the second half of the turning part pair up."""
    half = rot["dims"] // 2
    return _turn(x, positions, rot, lambda i: i, lambda i: i + half)


def attend(score, v, sink):
    """score (T, T) of one head, v (T, E): causal softmax whose denominator
    also holds exp(sink)."""
    T = score.shape[0]
    ahead = torch.ones(T, T, dtype=torch.bool).triu(1)
    score = score.masked_fill(ahead, -math.inf)
    m = torch.clamp(score.max(dim=1, keepdim=True).values, min=float(sink))
    w = torch.exp(score - m)
    return (w / (w.sum(dim=1, keepdim=True) + torch.exp(sink - m))) @ v


def latents(rows, weight, rank, rot, positions, eps):
    """rows (T, rank + rot) -> normed latents, the shared rotated key part."""
    return (norm(rows[:, :rank], weight, eps),
            rotate_pairs(rows[:, rank:], positions, rot))


def latent_attention(q, c, kr, uk, uv, sink, cfg, positions):
    """q (T, H * (dim + rot)) not rotated yet, c (T, rank), kr (T, rot)
    rotated -> (T, H * vdim)."""
    H, D, P, E = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"]
    T = q.shape[0]
    q = q.view(T, H, D + P)
    qr = rotate_pairs(q[..., D:], positions, cfg["rot"])
    k, v = (c @ uk.T).view(T, H, D), (c @ uv.T).view(T, H, E)
    out = []
    for h in range(H):
        s = q[:, h, :D] @ k[:, h].T + qr[:, h] @ kr.T
        out.append(attend(s * cfg["scale"], v[:, h], sink[h]))
    return torch.cat(out, dim=1)


def latent_mixer(W, p, h, cfg, eps):
    positions = range(h.shape[0])
    c, kr = latents(h @ W[p + "dkv"].T, W[p + "dkv.norm"], cfg["kv_rank"],
                    cfg["rot"], positions, eps)
    o = latent_attention(h @ W[p + "q"].T, c, kr, W[p + "uk"], W[p + "uv"],
                         W[p + "sink"], cfg, positions)
    return (o * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def retention(q, k, v, decay, state=None):
    """q, k (T, H, D), v (T, H, E), decay of H:  S <- decay S + k v^T,
    o = S^T q.  Returns (o, S (H, D, E))."""
    T, H, D = q.shape
    S = q.new_zeros(H, D, v.shape[2]) if state is None else state.clone()
    a = torch.tensor(decay, dtype=q.dtype).view(H, 1, 1)
    out = []
    for t in range(T):
        S = a * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
        out.append((S * q[t].unsqueeze(2)).sum(dim=1))
    return torch.stack(out), S


def retention_mixer(W, p, h, cfg, eps):
    H, D, E = cfg["heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    q = rotate_halves((h @ W[p + "q"].T).view(T, H, D), range(T), cfg["rot"])
    k = rotate_halves((h @ W[p + "k"].T).view(T, H, D), range(T), cfg["rot"])
    o, _ = retention(q, k * D ** -0.5, (h @ W[p + "v"].T).view(T, H, E),
                     cfg["decay"])
    o = rms(o, eps).reshape(T, H * E)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def poly_norm(z, act, eps):
    return act[0] * rms(z, eps) + act[1] * rms(z ** 2, eps) + \
        act[2] * rms(z ** 3, eps) + act[3]


def dense_mlp(W, p, h, cfg, eps, margins=None):
    return poly_norm(h @ W[p + "up"].T, W[p + "act"], eps) @ W[p + "down"].T


def _groups(r):
    g = r.get("groups") or {"count": 1, "keep": 1}
    return g["count"], g["keep"]


def route(z, count, keep, top):
    """Logits (T, experts) -> chosen experts and weights (T, top)."""
    e = torch.exp(z - z.max(dim=1, keepdim=True).values)
    s = e / e.sum(dim=1, keepdim=True)
    idx = []
    for row in s:
        parts = row.view(count, -1)
        n = parts.shape[1]
        score = [max(g.tolist()) for g in parts]
        best = sorted(range(count), key=lambda g: (-score[g], g))[:keep]
        may = sorted((j for g in best for j in range(g * n, g * n + n)),
                     key=lambda j: (-row[j].item(), j))
        idx.append(may[:top])
    idx = torch.tensor(idx)
    return idx, s.gather(1, idx)


def route_margin(z, count, keep, top):
    """How far every row's logits are from choosing otherwise: the smaller
    gap between the last kept and the first dropped group, or expert."""
    parts = z.view(len(z), count, -1)
    best, order = parts.amax(dim=2).sort(dim=1, descending=True)
    gap = torch.full((len(z),), math.inf, dtype=z.dtype)
    if keep < count:
        gap = best[:, keep - 1] - best[:, keep]
    open_ = torch.zeros_like(best, dtype=torch.bool).scatter_(
        1, order[:, :keep], True).repeat_interleave(parts.shape[2], dim=1)
    v = z.masked_fill(~open_, -math.inf).sort(dim=1, descending=True).values
    if top < z.shape[1]:
        gap = torch.minimum(gap, v[:, top - 1] - v[:, top])
    return gap


def expert(W, p, h):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def experts_mlp(W, p, h, cfg, eps, margins=None):
    r = cfg["router"]
    z = h @ W[p + "router"].T
    if margins is not None:
        margins.append(route_margin(z, *_groups(r), r["top"]))
    idx, w = route(z, *_groups(r), r["top"])
    out = torch.zeros_like(h)
    for e in range(r["experts"]):
        out += expert(W, f"{p}e{e}.", h) * \
            (w * (idx == e)).sum(dim=1, keepdim=True)
    if cfg.get("shared"):
        out += expert(W, p + "shared.", h)
    return out


def residual_gate(W, p, h):
    return sigmoid(h @ W[p].T + W[p + ".b"])


MIXERS = {"latent_attention": latent_mixer, "retention": retention_mixer}
MLPS = {"dense": dense_mlp, "moe": experts_mlp}


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None,
            margins=None):
    """Logits (T, vocab) of one sequence; ``layers`` collects the residual
    stream after every layer, ``margins`` the routers' margins."""
    W = {n: w.to(dtype) for n, w in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens)]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = norm(x, W[p + "norm1"], eps)
        y = MIXERS[L["type"]](W, p + "mix.", h, L["mixer"], eps)
        x = x + y * residual_gate(W, p + "rg1", h)
        if L["mlp"] is not None:
            y = MLPS[L["mlp"]["kind"]](W, p + "mlp.", h, L["mlp"], eps,
                                       margins)
            x = x + y * residual_gate(W, p + "rg2", h)
        if layers is not None:
            layers.append(x)
    return norm(x, W["final.norm"], eps) @ W["head"].T
