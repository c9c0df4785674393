"""Plain, slow implementation of the Voletar design for the tests.

One function per mechanism, one token after another, every weight used as
it is stored.  It shares no code with the package: sizes come from the
config dictionary, weights from a name -> tensor dictionary.  ``dtype`` is
the arithmetic (float64 for a golden answer, float32 to see rounding).
"""

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return rms(x, eps) * weight


def silu(x):
    return x / (1.0 + torch.exp(-x))


def log_sigmoid(x):
    # log(1 / (1 + e^-x)) without overflow on either side
    return torch.minimum(x, torch.zeros_like(x)) - torch.log1p(
        torch.exp(-x.abs()))


def relu_squared(x):
    return torch.clamp(x, min=0.0) ** 2


def visible(i, j, mask):
    """Does the query at position i see the key at position j?"""
    if j > i:
        return False
    if mask is None or mask.get("size") is None:
        return True
    return i - j < mask["size"] or j < mask.get("keep_first", 0)


def windowed_attention(q, k, v, scale, mask):
    """q (T, H, D), k (T, G, D), v (T, G, E) -> (T, H, E)."""
    T, H, _ = q.shape
    G = k.shape[1]
    keep = torch.tensor([[visible(i, j, mask) for j in range(T)]
                         for i in range(T)])
    out = q.new_zeros(T, H, v.shape[2])
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        s = s.masked_fill(~keep, -math.inf)
        w = torch.exp(s - s.max(dim=1, keepdim=True).values)
        out[:, h] = (w / w.sum(dim=1, keepdim=True)) @ v[:, g]
    return out


def decayed_memory(q, k, v, decay, state=None):
    """S <- decay S + k v^T, o = S^T q per head.  q, k (T, H, D),
    v (T, H, E), decay (H,).  Returns (o (T, H, E), S (H, D, E))."""
    T, H, D = q.shape
    S = q.new_zeros(H, D, v.shape[2]) if state is None else state.clone()
    out = []
    for t in range(T):
        S = decay.view(H, 1, 1) * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
        out.append((S * q[t].unsqueeze(2)).sum(dim=1))
    return torch.stack(out), S


def gated_memory(q, k, v, i_gate, f_gate, state=None):
    """The exponentially gated memory with its running maximum.
    q (already scaled), k (T, H, D), v (T, H, E), log gates (T, H).
    Returns (o (T, H, E), (S, n, m))."""
    T, H, D = q.shape
    if state is None:
        S = q.new_zeros(H, D, v.shape[2])
        n = q.new_zeros(H, D)
        m = q.new_zeros(H)
    else:
        S, n, m = (a.clone() for a in state)
    out = []
    for t in range(T):
        m_new = torch.maximum(f_gate[t] + m, i_gate[t])
        fs = torch.exp(f_gate[t] + m - m_new)
        ins = torch.exp(i_gate[t] - m_new)
        S = fs.view(H, 1, 1) * S + ins.view(H, 1, 1) * (
            k[t].unsqueeze(2) * v[t].unsqueeze(1))
        n = fs.view(H, 1) * n + ins.view(H, 1) * k[t]
        m = m_new
        num = (S * q[t].unsqueeze(2)).sum(dim=1)
        den = torch.maximum((n * q[t]).sum(dim=1).abs(), torch.exp(-m))
        out.append(num / (den + 1e-6).view(H, 1))
    return torch.stack(out), (S, n, m)


def lightning_mixer(W, p, h, cfg, eps):
    H, D, E = cfg["heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    q = silu(h @ W[p + "q"].T).view(T, H, D)
    k = silu(h @ W[p + "k"].T).view(T, H, D)
    v = silu(h @ W[p + "v"].T).view(T, H, E)
    decay = torch.tensor(cfg["decay"], dtype=h.dtype)
    o, _ = decayed_memory(q, k, v, decay)
    o = rms_norm(o.reshape(T, H * E), W[p + "norm"], eps)
    return (o * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def attention_branch(W, p, h, cfg):
    H, G, D, E = cfg["heads"], cfg["kv_heads"], cfg["dim"], cfg["vdim"]
    T = h.shape[0]
    o = windowed_attention((h @ W[p + "q"].T).view(T, H, D),
                           (h @ W[p + "k"].T).view(T, G, D),
                           (h @ W[p + "v"].T).view(T, G, E),
                           cfg["scale"], cfg.get("mask"))
    return o.reshape(T, H * E) @ W[p + "o"].T


def memory_branch(W, p, h, cfg, eps):
    H, D, E, cap = cfg["heads"], cfg["dim"], cfg["vdim"], cfg["gate_cap"]
    T = h.shape[0]
    q = (h @ W[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, D)
    v = (h @ W[p + "v"].T).view(T, H, E)
    i = cap * torch.tanh((h @ W[p + "i"].T + W[p + "i.b"]) / cap)
    f = log_sigmoid(
        cap * torch.tanh((h @ W[p + "f"].T + W[p + "f.b"]) / cap))
    o, _ = gated_memory(q, k, v, i, f)
    o = rms(o, eps).reshape(T, H * E) * W[p + "norm"]
    return (o * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def parallel_mixer(W, p, h, cfg, eps):
    a = attention_branch(W, p + "left.", h, cfg["left"])
    b = memory_branch(W, p + "right.", h, cfg["right"], eps)
    return 0.5 * (rms_norm(a, W[p + "left.out"], eps)
                  + rms_norm(b, W[p + "right.out"], eps))


MIXERS = {"lightning": lightning_mixer, "parallel": parallel_mixer}


def schedule(cfg):
    """(layer, pass or None) in the order they run; the pass is named at
    its first layer only."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    order = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        order += [(i, t if i == a else None) for i in range(a, b)]
    return order + [(i, None) for i in range(b, n)]


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits (T, vocab) of one sequence; ``layers`` collects the residual
    stream after every layer run."""
    W = {n: w.to(dtype) for n, w in weights.items()}
    eps = cfg["norm"]["eps"]
    x = x0 = W["embed"][torch.as_tensor(tokens)]
    for i, t in schedule(cfg):
        if t is not None:
            x = torch.cat([x, x0], dim=1) @ W["loop.in"].T + W["loop.step"][t]
        L, p = cfg["layers"][i], f"l{i}."
        h = rms_norm(x, W[p + "norm1"], eps)
        x = x + MIXERS[L["type"]](W, p + "mix.", h, L["mixer"], eps)
        if L["mlp"] is not None:
            h = rms_norm(x, W[p + "norm2"], eps)
            x = x + relu_squared(h @ W[p + "mlp.up"].T) @ W[p + "mlp.down"].T
        if layers is not None:
            layers.append(x)
    logits = rms_norm(x, W["final.norm"], eps) @ W["head"].T
    c = cfg["logit_softcap"]
    return c * torch.tanh(logits / c)
