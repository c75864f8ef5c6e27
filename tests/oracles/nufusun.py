"""Plain, slow reference of the Nufusun design on the CPU: one function per
mechanism, whole sequences only (no cache, no batching, no tiles), in the dtype
of the tensors it is given (float64 in the tests). It shares no code with
:mod:`kgs`; the tests compare the serving path with it.

``weights`` is a dict of tensors by their checkpoint names and ``cfg`` the
parsed ``config.json``.
"""
import math

import torch


def rms_norm(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * (1 + w)


def bucket(n, rows, far):
    """Row of the distance table for a key ``n`` tokens back: one row per distance
    up to half the table, then logarithmic up to distance ``far``."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * half + 1e-9))


def distance_bias(rel, far, T):
    """``[T, T, H]``: the bias of query i and key j <= i (zero elsewhere)."""
    rows = [bucket(n, rel.shape[0], far) for n in range(T)]
    by_n = rel[rows]
    out = torch.zeros(T, T, rel.shape[1], dtype=rel.dtype)
    for i in range(T):
        out[i, :i + 1] = by_n[:i + 1].flip(0)
    return out


def scores(q, k, scale, temp):
    """``q [T, H, D]``, ``k [T, G, D]`` -> ``[T, T, H]``, heads of one group in a row
    sharing a key head, each head at its own temperature."""
    H, G = q.shape[1], k.shape[1]
    return torch.stack([(q[:, h] @ k[:, h // (H // G)].T) * scale * temp[h] for h in range(H)], -1)


def talk(s, t):
    """Every head's score becomes a mixture of all heads' scores, ``t [H, H]``."""
    return s @ t.T


def softmax_plus_one(s):
    """Causal softmax over keys (dim 1) of ``[T, T, H]`` with one more term of score
    0 in the denominator."""
    T = s.shape[0]
    s = s.masked_fill(~torch.ones(T, T, dtype=torch.bool).tril()[..., None], -math.inf)
    m = torch.clamp(s.max(1, keepdim=True).values, min=0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(1, keepdim=True))


def attention(h, w, p, m):
    """The mixer of one layer, tensors ``p + name``."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]

    def lin(n, heads):
        return (h @ w[p + n].T + w[p + n + ".b"]).reshape(T, heads, -1)

    q, k, v = lin("q", H), lin("k", G), lin("v", G)
    s = scores(q, k, m["scale"], w[p + "temp"])
    s = talk(s + distance_bias(w[p + "rel"], m["bias_max"], T), w[p + "talk"])
    a = softmax_plus_one(s)
    o = torch.stack([a[..., x] @ v[:, x // (H // G)] for x in range(H)], 1)
    return o.reshape(T, -1) @ w[p + "o"].T + w[p + "o.b"]


def expert(h, gate, up, down, limit):
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ down.T


def route(h, router, top):
    """Chosen experts ``[T, top]`` and their weights (sigmoid scores as they are)."""
    s = torch.sigmoid(h @ router.T)
    return s.topk(top, -1).indices, s.topk(top, -1).values


def experts(h, w, p, m):
    """Mixture of experts; an expert's weight scales its input."""
    idx, weight = route(h, w[p + "router"], m["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), weight[t]):
            x = f"{p}e{e}."
            y[t] += expert(s * h[t], w[x + "gate"], w[x + "up"], w[x + "down"], m["expert"]["limit"])
    return y


def layer(x, w, i, entry, eps):
    """Mixer and feed-forward read the same normed input."""
    h = rms_norm(x, w[f"l{i}.norm1"], eps)
    y = attention(h, w, f"l{i}.mix.", entry["mixer"])
    if entry["mlp"] is not None:
        y = y + experts(h, w, f"l{i}.mlp.", entry["mlp"])
    return x + y


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits ``[T, vocab]``; ``layers``: a list that receives the residual after every layer."""
    w = {n: t.to(dtype) for n, t in weights.items()}
    x = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    for i, entry in enumerate(cfg["layers"]):
        x = layer(x, w, i, entry, cfg["norm"]["eps"])
        if layers is not None:
            layers.append(x)
    return rms_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T
