"""Plain, slow reference of the Nokipel design on the CPU: one function per
mechanism, whole sequences only (no cache, no batching, no tiles), in the dtype
of the tensors it is given (float64 in the tests). It shares no code with
:mod:`kgs`; the tests compare the serving path with it.

``weights`` is a dict of tensors by their checkpoint names and ``cfg`` the
parsed ``config.json``.
"""
import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    """RMS norm of equal consecutive parts, each by its own root mean square."""
    parts = x.reshape(*x.shape[:-1], groups, -1)
    return rms(parts, eps).reshape(x.shape) * w


def silu(z):
    return z * torch.sigmoid(z)


def rotate(x, dims, base):
    """``x [T, heads, dim]``: neighbouring pairs of the first ``dims`` dimensions turn
    by an angle per position (the row number) and pair."""
    T = x.shape[0]
    f = torch.tensor([base ** (-2 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    a = torch.arange(T, dtype=torch.float64)[:, None] * f[None]
    c, s = a.cos().to(x.dtype)[:, None], a.sin().to(x.dtype)[:, None]
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out = x.clone()
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def chunk_mask(T, size):
    """``[T, T]``: key j visible to query i (causal, same chunk of positions)."""
    p = torch.arange(T)
    return (p[None] <= p[:, None]) & (p[None] // size == p[:, None] // size)


def attention(h, w, p, m):
    """The attention mixer of one layer, tensors ``p + name``."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]

    def lin(n, heads):
        return (h @ w[p + n].T + w[p + n + ".b"]).reshape(T, heads, -1)

    q, k, v = lin("q", H), lin("k", G), lin("v", G)
    q, k = (rotate(x, m["rot"]["dims"], m["rot"]["base"]) for x in (q, k))
    mask = chunk_mask(T, m["mask"]["size"])
    out = []
    for x in range(H):
        g = x // (H // G)
        s = (q[:, x] @ k[:, g].T * m["scale"]).masked_fill(~mask, -math.inf)
        out.append(torch.softmax(s, -1) @ v[:, g])
    return torch.cat(out, -1) @ w[p + "o"].T


def recurrence(q, k, v, decay):
    """``S <- decay S + k v^T; o = S^T q`` per head; ``[T, H, *]`` in, ``[T, H, V]`` out."""
    T, H = q.shape[:2]
    d = torch.tensor(decay, dtype=q.dtype)[:, None, None]
    S = torch.zeros(H, k.shape[2], v.shape[2], dtype=q.dtype)
    o = []
    for t in range(T):
        S = d * S + k[t][:, :, None] * v[t][:, None, :]
        o.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(o)


def lightning(h, w, p, m, eps):
    T, H = h.shape[0], m["heads"]
    q, k, v = (silu(h @ w[p + n].T).reshape(T, H, -1) for n in "qkv")
    o = recurrence(q, k, v, m["decay"]).reshape(T, -1)
    return (rms(o, eps) * w[p + "norm"] * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def dense(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ w[p + "down"].T


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, router, correction, m):
    """Chosen outputs and their weights, ``[T, top]`` each."""
    s = torch.softmax(h @ router.T, -1)
    choice = s + correction
    if m.get("groups"):
        n, keep = m["groups"]["count"], m["groups"]["keep"]
        parts = choice.reshape(len(h), n, -1)
        best = parts.max(-1).values.topk(keep, -1).indices
        kept = torch.zeros(len(h), n, dtype=torch.bool).scatter(1, best, True)
        choice = parts.masked_fill(~kept[..., None], -math.inf).reshape(choice.shape)
    idx = choice.topk(m["top"], -1).indices
    chosen = s.gather(1, idx)
    return idx, chosen / (chosen.sum(-1, keepdim=True) + 1e-20) * m.get("scale", 1.0)


def experts(h, w, p, m):
    idx, weight = route(h, w[p + "router"], w[p + "correction"], m["router"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in zip(idx[t].tolist(), weight[t]):
            y[t] += s * (expert(h[t], w, f"{p}e{e}.") if e < m["router"]["experts"] else h[t])
    if m.get("shared"):
        y = y + torch.sigmoid(h @ w[p + "shared.sg"].T) * expert(h, w, p + "shared.")
    return y


def layer(x, w, i, entry, norm):
    p, n = f"l{i}.", (norm["groups"], norm["eps"])
    h = group_norm(x, w[p + "norm1"], *n)
    if entry["type"] == "attention":
        x = x + attention(h, w, p + "mix.", entry["mixer"])
    else:
        x = x + lightning(h, w, p + "mix.", entry["mixer"], norm["eps"])
    if entry["mlp"] is not None:
        h = group_norm(x, w[p + "norm2"], *n)
        if entry["mlp"]["kind"] == "dense":
            x = x + dense(h, w, p + "mlp.", entry["mlp"]["limit"])
        else:
            x = x + experts(h, w, p + "mlp.", entry["mlp"])
    return x


def order(cfg):
    """``(layer, embedding output added before it)`` of every layer run."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b = lp["start"], lp["stop"]
    runs = [(i, False) for i in range(a)]
    for t in range(lp["times"]):
        runs += [(i, t > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits ``[T, vocab]``; ``layers``: a list that receives the residual after every layer run."""
    w = {n: t.to(dtype) for n, t in weights.items()}
    x0 = w["embed"][torch.as_tensor(tokens)] * cfg["embedding"]["scale"]
    x = x0
    for i, again in order(cfg):
        x = layer(x + x0 if again else x, w, i, cfg["layers"][i], cfg["norm"])
        if layers is not None:
            layers.append(x)
    return group_norm(x, w["final.norm"], cfg["norm"]["groups"], cfg["norm"]["eps"]) @ w["head"].T
