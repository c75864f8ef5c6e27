"""Small Vumalix configurations and weights for the tests, and runs of the oracle on them.
Together they cover every branch: both mixers with and without a feed-forward, layers with
another layer's weights (an earlier or a later one's), windows from one key to more than
the prompts have, convolutions of one tap (no state), two, four and seven, groups of one to
forty heads, and sizes that the MFMA kernels take, pad or leave to the plain ones."""
import torch

from kgs.models.vumalix import VumalixConfig, random_weights


def latent(heads, dim, rot, vdim, q_rank, kv_rank, window, base, scale, ff=None, of=None):
    e = {"type": "latent_attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
         "mixer": {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
                   "mask": {"size": window}, "rot": {"dims": rot, "base": base}}}
    return e if of is None else {**e, "weights_of": of}


def attention(heads, kv_heads, dim, vdim, scale, diff, temp, ff=None, of=None):
    e = {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
         "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff,
                   "q_temp": {"coef": temp[0], "every": temp[1]}}}
    return e if of is None else {**e, "weights_of": of}


_L = (3, 24, 8, 40, 36, 56, 20, 1e3, 0.25, 72)
_A = (4, 2, 24, 40, 0.2, 0.3, (0.5, 7), 100)
_P = (6, 48, 12, 48, 40, 100, 45, 30.0, 0.2, 40)
MODELS = {
    "mixed": dict(vocab=203, width=140, canon={"taps": 4}, norm={"eps": 3e-6}, layers=[
        latent(*_L), attention(*_A), latent(*_L, of=0), attention(5, 5, 16, 64, 0.3, -0.2, (0.2, 33)), attention(*_A, of=1),
        latent(*_L, of=0)]),
    "edges": dict(vocab=131, width=192, canon={"taps": 2}, norm={"eps": 1e-5}, layers=[
        attention(12, 3, 64, 128, 0.15, 0.8, (0.6, 64), 200), latent(16, 64, 64, 64, 80, 130, 33, 1e4, 0.1),
        latent(3, 100, 32, 128, 96, 512, 64, 5e5, 0.15, 64), latent(2, 32, 2, 64, 24, 64, 1, 10.0, 0.5, 130)]),
    # no state: one tap
    "stateless": dict(vocab=97, width=256, canon={"taps": 1}, norm={"eps": 1e-4}, layers=[
        attention(8, 1, 128, 64, 0.2, 0.5, (0.1, 1), 256), latent(4, 64, 16, 64, 64, 64, 1000, 1e4, 0.2, 96),
        attention(40, 1, 40, 100, 0.3, 0.0, (0.0, 9), 48)]),
    # beyond the MFMA kernels' sizes; the weights of a later layer
    "large": dict(vocab=150, width=320, canon={"taps": 7}, norm={"eps": 1e-5}, layers=[
        latent(2, 160, 96, 48, 64, 600, 40, 1e5, 0.08, 64), latent(*_P, of=2), latent(*_P),
        attention(6, 3, 160, 80, 0.12, 0.6, (0.3, 16), 72)]),
}


def config(name: str) -> VumalixConfig:
    return VumalixConfig.from_dict({"architecture": "Vumalix", **MODELS[name]})


def weights(cfg: VumalixConfig, seed: int = 0) -> dict:
    """Random weights whose lambdas are far from 0 and whose convolutions matter."""
    w = random_weights(cfg, seed)
    for name in w:
        f = 1.5 if name.rsplit(".", 1)[-1] in ("lq1", "lk1", "lq2", "lk2", "uq", "canon1") else 1
        w[name] = (w[name].float() * f).to(torch.bfloat16)
    return w


def model(name: str):
    cfg = config(name)
    return cfg, weights(cfg)


_CACHE: dict = {}


def oracle_logits(name: str, tokens) -> torch.Tensor:
    """float64 logits of every position (prefixes of longer runs are reused)."""
    from oracles import vumalix as O

    if name not in _CACHE:
        cfg, w = model(name)
        _CACHE[name] = (cfg.raw, w, {})
    raw, w, runs = _CACHE[name]
    tokens = tuple(int(t) for t in tokens)
    for done, logits in runs.items():
        if done[:len(tokens)] == tokens:
            return logits[:len(tokens)]
    with torch.no_grad():
        runs[tokens] = O.forward(raw, w, list(tokens))
    return runs[tokens]
