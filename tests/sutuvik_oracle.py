"""Plain, slow implementation of the Sutuvik design for the tests.

One function per mechanism, every weight used as it is stored, recurrences one
token after another.  It shares no code with the package: sizes come from the
config dictionary, weights from a name -> tensor dictionary.  ``dtype`` is the
arithmetic (float64 for a golden answer, float32 to see rounding).
"""

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def group_norm(x, weight, groups, eps):
    """Every one of ``groups`` equal parts over its own root mean square."""
    T, W = x.shape
    return rms(x.reshape(T, groups, W // groups), eps).reshape(T, W) * weight


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def causal_conv(x, w):
    """x (T, C), w (C, taps): the last column weighs the row itself."""
    taps = w.shape[1]
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] += w[:, j] * x[s]
    return out


def frequency(i, rot):
    """Radians a position of pair i, after the scaling of long wavelengths."""
    f = rot["base"] ** (-2.0 * i / rot["dims"])
    sc = rot.get("scaling")
    if not sc:
        return f
    wave = 2.0 * math.pi / f
    if wave < sc["original"] / sc["high"]:
        return f
    if wave > sc["original"] / sc["low"]:
        return f / sc["factor"]
    s = (sc["original"] / wave - sc["low"]) / (sc["high"] - sc["low"])
    return (1.0 - s) * f / sc["factor"] + s * f


def rotate_pairs(x, positions, rot):
    """x (T, heads, n): elements 2i and 2i + 1 of the first dims turn."""
    out = x.clone()
    p = torch.tensor([float(p) for p in positions], dtype=torch.float64)
    for i in range(rot["dims"] // 2):
        a = p * frequency(i, rot)
        c, s = (f(a).to(x.dtype)[:, None] for f in (torch.cos, torch.sin))
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def query_temperature(p, coef, every):
    return 1.0 + coef * math.log((p + 1) // every + 1)


def slope(h, heads):
    return 2.0 ** (-8.0 * (h + 1) / heads)


def attend(score, v, sink):
    """score (T, T) of one head, v (T, E): causal softmax whose denominator
    also holds exp(sink)."""
    T = score.shape[0]
    ahead = torch.ones(T, T, dtype=torch.bool).triu(1)
    score = score.masked_fill(ahead, -math.inf)
    m = torch.clamp(score.max(dim=1, keepdim=True).values, min=float(sink))
    w = torch.exp(score - m)
    return (w / (w.sum(dim=1, keepdim=True) + torch.exp(sink - m))) @ v


def mixed_values(v, lam, first):
    return v if first is None else (1.0 - lam) * v + lam * first


def biased_attention(W, p, h, cfg, eps, first):
    """Normed queries and keys, a query temperature, a distance bias, a
    learned sink and a gate a head.  Returns (output, own values)."""
    H, G, D, E = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    q = rms((h @ W[p + "q"].T).view(T, H, D), eps) * W[p + "q.norm"]
    k = rms((h @ W[p + "k"].T).view(T, G, D), eps) * W[p + "k.norm"]
    raw = h @ W[p + "v"].T
    v = raw if not cfg.get("v_mix") else mixed_values(
        raw, W[p + "vmix"], first)
    v = v.view(T, G, E)
    t = cfg["q_temp"]
    q = q * torch.tensor([query_temperature(i, t["coef"], t["every"])
                          for i in range(T)], dtype=h.dtype).view(T, 1, 1)
    pos = torch.arange(T, dtype=h.dtype)
    far = pos[:, None] - pos[None, :]
    gate = sigmoid(h @ W[p + "g"].T)
    out = []
    for i in range(H):
        g = i // (H // G)
        s = (q[:, i] @ k[:, g].T) * cfg["scale"] - slope(i, H) * far
        out.append(attend(s, v[:, g], W[p + "sink"][i]) * gate[:, i:i + 1])
    return torch.cat(out, dim=1) @ W[p + "o"].T, raw


def capped_attention(W, p, h, cfg, eps, first):
    """Rotated, then normed queries and keys; scores times a number a head,
    soft-capped; one added to the denominator."""
    H, G, D, E = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    q = rms(rotate_pairs((h @ W[p + "q"].T).view(T, H, D), range(T),
                         cfg["rot"]), eps)
    k = rms(rotate_pairs((h @ W[p + "k"].T).view(T, G, D), range(T),
                         cfg["rot"]), eps)
    raw = h @ W[p + "v"].T
    v = raw if not cfg.get("v_mix") else mixed_values(
        raw, W[p + "vmix"], first)
    v = v.view(T, G, E)
    c, zero = cfg["softcap"], torch.zeros((), dtype=h.dtype)
    out = []
    for i in range(H):
        g = i // (H // G)
        s = (q[:, i] @ k[:, g].T) * cfg["scale"] * W[p + "temp"][i]
        out.append(attend(c * torch.tanh(s / c), v[:, g], zero))
    return torch.cat(out, dim=1) @ W[p + "o"].T, raw


def state_space(x, B, C, dt, decay, skip, state=None):
    """x (T, H, P), B, C (T, G, N), dt (T, H), decay (T, H):
    S <- decay S + dt B x^T, y = S^T C + skip x.  Returns (y, S (H, N, P))."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    S = x.new_zeros(H, N, P) if state is None else state.clone()
    of = [h // (H // G) for h in range(H)]
    out = []
    for t in range(T):
        S = decay[t].view(H, 1, 1) * S + dt[t].view(H, 1, 1) * (
            B[t][of].unsqueeze(2) * x[t].unsqueeze(1))
        out.append((S * C[t][of].unsqueeze(2)).sum(dim=1)
                   + skip.view(H, 1) * x[t])
    return torch.stack(out), S


def mamba2_mixer(W, p, h, cfg, eps):
    H, P, N, G = cfg["heads"], cfg["vdim"], cfg["state"], cfg["groups"]
    T, inner = h.shape[0], H * P
    z, c, dt = (h @ W[p + "in"].T).split([inner, inner + 2 * G * N, H], dim=1)
    c = silu(causal_conv(c, W[p + "conv"]) + W[p + "conv.b"])
    x, B, C = c.split([inner, G * N, G * N], dim=1)
    dt = softplus(dt + W[p + "dt_bias"])
    y, _ = state_space(x.view(T, H, P), B.view(T, G, N), C.view(T, G, N), dt,
                       torch.exp(-torch.exp(W[p + "A_log"]) * dt), W[p + "D"])
    y = group_norm(y.reshape(T, inner) * silu(z), W[p + "norm"],
                   cfg["norm_groups"], eps)
    return y @ W[p + "o"].T


def route(z, correction, groups, keep, top):
    """Logits (T, experts) -> chosen experts and weights (T, top)."""
    s = sigmoid(z)
    idx = []
    for row in s + correction:
        parts = row.view(groups, -1)
        score = [sum(sorted(g.tolist(), reverse=True)[:2]) for g in parts]
        best = sorted(range(groups), key=lambda g: (-score[g], g))[:keep]
        n = parts.shape[1]
        may = sorted((e for g in best for e in range(g * n, g * n + n)),
                     key=lambda e: (-row[e].item(), e))
        idx.append(may[:top])
    idx = torch.tensor(idx)
    w = s.gather(1, idx)
    return idx, w / (w.sum(dim=1, keepdim=True) + 1e-20)


def route_margin(z, correction, groups, keep, top):
    """How far every row is from choosing otherwise: the smaller gap between
    the last kept and the first dropped group, or expert."""
    s = sigmoid(z) + correction
    parts = s.view(len(s), groups, -1)
    n = min(2, parts.shape[2])
    score = parts.sort(dim=2, descending=True).values[..., :n].sum(dim=2)
    best, order = score.sort(dim=1, descending=True)
    gap = torch.full((len(s),), math.inf, dtype=s.dtype)
    if keep < groups:
        gap = best[:, keep - 1] - best[:, keep]
    open_ = torch.zeros_like(score, dtype=torch.bool).scatter_(
        1, order[:, :keep], True).repeat_interleave(parts.shape[2], dim=1)
    v = s.masked_fill(~open_, -math.inf).sort(dim=1, descending=True).values
    if top < s.shape[1]:
        gap = torch.minimum(gap, v[:, top - 1] - v[:, top])
    return gap


def experts_mlp(W, p, h, cfg, margins=None):
    r = cfg["router"]
    if margins is not None:
        margins.append(route_margin(
            h @ W[p + "router"].T, W[p + "correction"], r["groups"]["count"],
            r["groups"]["keep"], r["top"]))
    idx, w = route(h @ W[p + "router"].T, W[p + "correction"],
                   r["groups"]["count"], r["groups"]["keep"], r["top"])
    out = torch.zeros_like(h)
    for e in range(r["experts"]):
        q = f"{p}e{e}."
        y = (silu(h @ W[q + "gate"].T) * (h @ W[q + "up"].T)) @ W[q + "down"].T
        out += y * (w * (idx == e)).sum(dim=1, keepdim=True)
    return out


def token_side(W, p, x, e, eps):
    """The layer's own row of the token, gated by the stream."""
    y = (gelu_tanh(x @ W[p + "gate"].T) * e) @ W[p + "proj"].T
    return rms(y, eps) * W[p + "norm"]


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None,
            margins=None):
    """Logits (T, vocab) of one sequence; ``layers`` collects the residual
    stream after every layer, ``margins`` the routers' margins."""
    W = {n: w.to(dtype) for n, w in weights.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    dim = cfg["token_side"]["dim"]
    toks = torch.as_tensor(tokens)
    x = group_norm(W["embed"][toks], W["embed.norm"], groups, eps)
    first = None
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        h = group_norm(x, W[p + "norm1"], groups, eps)
        h = h + causal_conv(h, W[p + "canon1"])
        if L["type"] == "mamba2":
            y = mamba2_mixer(W, p + "mix.", h, m, eps)
        else:
            f = {"attention": biased_attention,
                 "attention_2": capped_attention}[L["type"]]
            y, own = f(W, p + "mix.", h, m, eps, first)
            if m.get("v_mix") and first is None:
                first = own
        x = x + y
        if L["mlp"] is not None:
            h = group_norm(x, W[p + "norm2"], groups, eps)
            x = x + experts_mlp(W, p + "mlp.", h, L["mlp"], margins)
        e = W["side.embed"][toks][:, i * dim:(i + 1) * dim]
        x = x + token_side(W, p + "side.", x, e, eps)
        if layers is not None:
            layers.append(x)
    x = group_norm(x, W["final.norm"], groups, eps)
    return x @ W["embed"].T * cfg["logit_scale"]
