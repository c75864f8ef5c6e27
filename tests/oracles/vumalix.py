"""Plain, slow reference of the Vumalix design on the CPU: one function per
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


def causal_conv(x, w):
    """``x [T, D]``, ``w [D, taps]``: every channel by itself, the last tap on the row
    itself, zeros before the first row."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=x.dtype), x])
    return sum(w[:, j] * padded[j:j + x.shape[0]] for j in range(taps))


def rotate_half(x, base):
    """``x [T, heads, dims]``: dimension i turns with dimension i + dims / 2 by an angle per
    position (the row number) and pair."""
    T, dims = x.shape[0], x.shape[-1]
    half = dims // 2
    f = torch.tensor([base ** (-2 * i / dims) for i in range(half)], dtype=torch.float64)
    a = torch.arange(T, dtype=torch.float64)[:, None] * f[None]
    c, s = a.cos().to(x.dtype)[:, None], a.sin().to(x.dtype)[:, None]
    u, v = x[..., :half], x[..., half:]
    return torch.cat([u * c - v * s, v * c + u * s], -1)


def window_mask(T, size):
    """``[T, T]``: key j visible to query i (itself and the size - 1 keys before it)."""
    d = torch.arange(T)[:, None] - torch.arange(T)[None]
    return (d >= 0) & (d < size)


def weighted(scores, mask, v):
    return torch.softmax(scores.masked_fill(~mask, -math.inf), -1) @ v


def latent_attention(h, w, p, m, eps):
    T, H, d, r, n = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    q = ((rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]) @ w[p + "uq"].T).reshape(T, H, d + r)
    z = h @ w[p + "dkv"].T
    c = rms(z[:, :n], eps) * w[p + "dkv.norm"]
    kr = rotate_half(z[:, None, n:], m["rot"]["base"])[:, 0]
    qr = rotate_half(q[..., d:], m["rot"]["base"])
    k, v = (c @ w[p + "uk"].T).reshape(T, H, d), (c @ w[p + "uv"].T).reshape(T, H, -1)
    mask = window_mask(T, m["mask"]["size"])
    out = [weighted((q[:, x, :d] @ k[:, x].T + qr[:, x] @ kr.T) * m["scale"], mask, v[:, x]) for x in range(H)]
    return (torch.cat(out, -1) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def temperature(T, m, dtype):
    """The factor of every position's queries."""
    return torch.tensor([1 + m["coef"] * math.log((p + 1) // m["every"] + 1) for p in range(T)], dtype=dtype)


def mixing_lambda(w, p, diff):
    return torch.exp((w[p + "lq1"] * w[p + "lk1"]).sum()) - torch.exp((w[p + "lq2"] * w[p + "lk2"]).sum()) + diff


def differential_attention(h, w, p, m, eps):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q = rms((h @ w[p + "q"].T).reshape(T, H, 2, d), eps) * w[p + "q.norm"]
    k = rms((h @ w[p + "k"].T).reshape(T, G, 2, d), eps) * w[p + "k.norm"]
    v = (h @ w[p + "v"].T).reshape(T, G, -1)
    q = q * temperature(T, m["q_temp"], h.dtype)[:, None, None, None]
    mask, lam = window_mask(T, T), mixing_lambda(w, p, m["diff"])
    out = []
    for x in range(H):
        g = x // (H // G)
        a1, a2 = (weighted(q[:, x, i] @ k[:, g, i].T * m["scale"], mask, v[:, g]) for i in range(2))
        out.append(rms(a1 - lam * a2, eps) * (1 - m["diff"]))
    return torch.cat(out, -1) @ w[p + "o"].T


def poly_norm(z, act, eps):
    a, b, c, e = act
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def dense(x, w, p, eps):
    return poly_norm(x @ w[p + "up"].T, w[p + "act"], eps) @ w[p + "down"].T


MIXERS = {"latent_attention": latent_attention, "attention": differential_attention}


def layer(x, w, i, entry, eps):
    p = f"l{entry.get('weights_of', i)}."
    h = x + causal_conv(x, w[p + "canon1"])
    x = x + rms(MIXERS[entry["type"]](h, w, p + "mix.", entry["mixer"], eps), eps) * w[p + "norm1"]
    if entry["mlp"] is not None:
        x = x + rms(dense(x, w, p + "mlp.", eps), eps) * w[p + "norm2"]
    return x


def forward(cfg, weights, tokens, dtype=torch.float64, layers=None):
    """Logits ``[T, vocab]``; ``layers``: a list that receives the residual after every layer."""
    w = {n: t.to(dtype) for n, t in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)]
    for i, entry in enumerate(cfg["layers"]):
        x = layer(x, w, i, entry, eps)
        if layers is not None:
            layers.append(x)
    return rms(x, eps) * w["final.norm"] @ w["head"].T
