"""Plain, slow implementation of the Nesilorn design for the tests.

One function per mechanism, every weight used as it is stored.  It shares no
code with the package: sizes come from the config dictionary, weights from a
name -> tensor dictionary.  ``dtype`` is the arithmetic (float64 for a golden
answer, float32 to see rounding).
"""

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def centred_norm(x, weight, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1.0 + weight)


def plain_norm(x, weight, eps):
    return rms(x, eps) * weight


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rotate(x, positions, base):
    """x (T, ..., n): element i turns with element i + n/2 by the angle
    position * base^(-2i/n)."""
    n = x.shape[-1]
    out = x.clone()
    for t, p in enumerate(positions):
        for i in range(n // 2):
            a = p * base ** (-2.0 * i / n)
            c, s = math.cos(a), math.sin(a)
            u, v = x[t, ..., i], x[t, ..., i + n // 2]
            out[t, ..., i] = u * c - v * s
            out[t, ..., i + n // 2] = v * c + u * s
    return out


def visible(i, j, size):
    """Does the query at position i see the key at position j?  size None:
    no window."""
    return 0 <= i - j and (size is None or i - j < size)


def window_attention(q, k, v, scale, size):
    """q, k (T, H, D), v (T, H, E) -> (T, H, E)."""
    T, H, _ = q.shape
    keep = torch.tensor([[visible(i, j, size) for j in range(T)]
                         for i in range(T)])
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h].T) * scale
        s = s.masked_fill(~keep, -math.inf)
        w = torch.exp(s - s.max(dim=1, keepdim=True).values)
        out.append((w / w.sum(dim=1, keepdim=True)) @ v[:, h])
    return torch.stack(out, dim=1)


def latents(rows, norm, kv_rank, base, positions, eps):
    """rows (T, kv_rank + rot) -> normed latents, rotated shared keys."""
    return (plain_norm(rows[:, :kv_rank], norm, eps),
            rotate(rows[:, kv_rank:], positions, base))


def latent_attention(q, c, kr, uk, uv, cfg, positions):
    """q (T, H*(dim + rot)) not rotated yet, c (T, rank), kr (T, rot)
    rotated -> (T, H*vdim)."""
    H, D, R, E = cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"]
    T = q.shape[0]
    q = q.view(T, H, D + R)
    q = torch.cat([q[..., :D],
                   rotate(q[..., D:], positions, cfg["rot"]["base"])], -1)
    k = torch.cat([(c @ uk.T).view(T, H, D),
                   kr.view(T, 1, R).expand(T, H, R)], -1)
    v = (c @ uv.T).view(T, H, E)
    mask = cfg.get("mask") or {}
    return window_attention(q, k, v, cfg["scale"],
                            mask.get("size")).reshape(T, H * E)


def latent_mixer(W, p, h, cfg, eps):
    positions = range(h.shape[0])
    c, kr = latents(h @ W[p + "dkv"].T, W[p + "dkv.norm"], cfg["kv_rank"],
                    cfg["rot"]["base"], positions, eps)
    o = latent_attention(h @ W[p + "q"].T, c, kr, W[p + "uk"], W[p + "uv"],
                         cfg, positions)
    return (o * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def route(z, top):
    """Logits (T, experts) -> chosen experts and weights (T, top)."""
    val, idx = torch.sort(z, dim=1, descending=True, stable=True)
    val, idx = val[:, :top], idx[:, :top]
    w = torch.exp(val - val[:, :1])
    return idx, w / w.sum(dim=1, keepdim=True)


def clamped_glu(gate, up, limit):
    g = torch.minimum(gate, torch.full_like(gate, limit))
    u = up.clamp(-limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def expert(W, p, h, limit):
    return clamped_glu(h @ W[p + "gate"].T, h @ W[p + "up"].T,
                       limit) @ W[p + "down"].T


def experts_mlp(W, p, h, cfg):
    idx, w = route(h @ W[p + "router"].T + W[p + "router.b"],
                   cfg["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(cfg["router"]["experts"]):
        y = expert(W, f"{p}e{e}.", h, cfg["expert"]["limit"])
        out += y * (w * (idx == e)).sum(dim=1, keepdim=True)
    return out


def dense_mlp(W, p, h, cfg):
    return gelu_tanh(h @ W[p + "up"].T) @ W[p + "down"].T


MIXERS = {"latent_attention": latent_mixer}
MLPS = {"dense": dense_mlp, "moe": experts_mlp}


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits (T, vocab) of one sequence; ``layers`` collects the residual
    stream after every layer."""
    W = {n: w.to(dtype) for n, w in weights.items()}
    eps = cfg["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        y = MIXERS[L["type"]](W, p + "mix.", x, L["mixer"], eps)
        x = x + centred_norm(y, W[p + "norm1"], eps)
        if L["mlp"] is not None:
            y = MLPS[L["mlp"]["kind"]](W, p + "mlp.", x, L["mlp"])
            x = x + centred_norm(y, W[p + "norm2"], eps)
        if layers is not None:
            layers.append(x)
    return centred_norm(x, W["final.norm"], eps) @ W["embed"].T
