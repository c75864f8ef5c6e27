"""Plain, slow reference of the Ruruzen design on the CPU: one function per
mechanism, whole sequences only (no cache, no batching, no chunking), in the
dtype of the tensors it is given (float64 in the tests). It shares no code with
:mod:`kgs`; the tests compare the serving path with it.

``weights`` is a dict of tensors by their checkpoint names and ``cfg`` the
parsed ``config.json``.
"""
import math

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def hyper_in(streams, w_in):
    """Read-out of the parallel residual streams: ``[T, S, D] -> [T, D]``."""
    return sum(w_in[s] * streams[:, s] for s in range(streams.shape[1]))


def hyper_out(streams, y, mix, w_out):
    """Every stream from all the old ones (``mix[from, to]``) plus its share of ``y``."""
    s = streams.shape[1]
    return torch.stack([sum(mix[f, t] * streams[:, f] for f in range(s)) + w_out[t] * y for t in range(s)], 1)


def short_conv(x, w):
    """Causal depthwise convolution ``[T, C]`` with ``w [C, taps]`` (last column:
    the current token), zeros before the start, no activation."""
    taps = w.shape[1]
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                out[t] += w[:, j] * x[src]
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(q, k, v, g, beta, state=None):
    """Gated delta rule with one decay per key channel. ``q, k, g [T, H, K]``,
    ``v [T, H, V]``, ``beta [T, H]`` -> ``(o [T, H, V], state [H, K, V])``."""
    T, H, K = q.shape
    S = torch.zeros(H, K, v.shape[-1], dtype=q.dtype) if state is None else state.clone()
    o = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            Sh = g[t, h][:, None] * S[h]
            u = beta[t, h] * (v[t, h] - Sh.T @ k[t, h])
            Sh = Sh + k[t, h][:, None] * u[None, :]
            S[h] = Sh
            o[t, h] = Sh.T @ q[t, h]
    return o, S


def causal_softmax_attention(q, k, v, scale):
    """``q, k [T, H, d]``, ``v [T, H, dv]`` -> ``[T, H, dv]``."""
    T = q.shape[0]
    s = torch.einsum("thd,jhd->htj", q, k) * scale
    mask = torch.arange(T)[None, :] <= torch.arange(T)[:, None]
    s = s.masked_fill(~mask, float("-inf"))
    return torch.einsum("htj,jhv->thv", torch.softmax(s, -1), v)


def latent(h, w, pre, eps):
    """The normalised latent a layer caches."""
    return rms_norm(h @ w[pre + "dkv"].T, w[pre + "dkv.norm"], eps)


def latent_attention(h, c, w, pre, m, eps):
    """``c``: the layer's own latent, or the one of the layer it reads."""
    T, H = h.shape[0], m["heads"]
    cq = rms_norm(h @ w[pre + "dq"].T, w[pre + "dq.norm"], eps)
    q = (cq @ w[pre + "uq"].T).reshape(T, H, m["dim"])
    k = (c @ w[pre + "uk"].T).reshape(T, H, m["dim"])
    v = (c @ w[pre + "uv"].T).reshape(T, H, m["vdim"])
    o = causal_softmax_attention(q, k, v, m["scale"])
    o = o * torch.sigmoid(h @ w[pre + "g"].T)[:, :, None]
    return o.reshape(T, -1) @ w[pre + "o"].T


def channel_delta(h, w, pre, m, eps):
    T, H, G, K, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(short_conv(h @ w[pre + n].T, w[pre + n + ".conv"])) for n in "qkv")
    rep = H // G
    q = (unit(q.reshape(T, G, K)) * K ** -0.5).repeat_interleave(rep, 1)
    k = unit(k.reshape(T, G, K)).repeat_interleave(rep, 1)
    beta = torch.sigmoid(h @ w[pre + "b"].T)
    a = ((h @ w[pre + "a1"].T) @ w[pre + "a2"].T + w[pre + "dt_bias"]).reshape(T, H, K)
    g = torch.exp(-torch.exp(w[pre + "A_log"])[None, :, None] * softplus(a))
    o, _ = delta_rule(q, k, v.reshape(T, H, V), g, beta)
    o = rms_norm(o, w[pre + "norm"], eps)
    o = o * torch.sigmoid((h @ w[pre + "g1"].T) @ w[pre + "g2"].T).reshape(T, H, V)
    return o.reshape(T, -1) @ w[pre + "o"].T


def dense_ff(h, w, pre):
    return (gelu_tanh(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def forward(cfg, w, tokens, residuals=None):
    """Logits ``[T, vocab]`` of one sequence. ``residuals``: a list that collects
    the sum of the streams after every layer."""
    eps, S = cfg["norm"]["eps"], cfg["streams"]
    x = rms_norm(w["embed"][torch.as_tensor(tokens)], w["embed.norm"], eps)
    streams = x[:, None, :].repeat(1, S, 1)
    latents = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]

        def sub(q, fn):
            hc = f"{p}hc{q}."
            h = rms_norm(hyper_in(streams, w[hc + "in"]), w[f"{p}norm{q}"], eps)
            return hyper_out(streams, fn(h), w[hc + "mix"], w[hc + "out"])

        def mixer(h):
            if layer["type"] == "channel_delta":
                return channel_delta(h, w, p + "mix.", m, eps)
            src = m.get("kv_from", i)
            if src == i:
                latents[i] = latent(h, w, p + "mix.", eps)
            return latent_attention(h, latents[src], w, p + "mix.", m, eps)

        streams = sub(1, mixer)
        if layer["mlp"] is not None:
            streams = sub(2, lambda h: dense_ff(h, w, p + "mlp."))
        if residuals is not None:
            residuals.append(streams.sum(1))
    logits = rms_norm(streams.sum(1), w["final.norm"], eps) @ w["embed"].T
    cap = cfg["logit_softcap"]
    return cap * torch.tanh(logits / cap)
