"""Small Ruruzen configurations and weights for the tests, and runs of the oracle
on them. No two mechanisms' sizes coincide by accident within one model unless a
case says so."""
import torch

from kgs.models.ruruzen import RuruzenConfig, random_weights


def latent(heads, dim, vdim, q_rank, kv_rank, scale, ff=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def delta(heads, kv_heads, dim, vdim, conv, ff=None):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                               "conv": conv},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


MODELS = {
    # delta first (no latent before it), shared latent over a delta layer, unequal dims
    "odd": dict(vocab=203, width=140, streams=3, logit_softcap=12.5, norm={"eps": 3e-6}, layers=[
        delta(6, 2, 20, 28, 3, ff=90), latent(5, 24, 40, 44, 72, 0.31, ff=200),
        delta(3, 3, 36, 12, 2), latent(3, 56, 16, 20, 72, 0.09, kv_from=1), latent(2, 16, 16, 36, 40, 0.5)]),
    # one stream, one head, taps 1 (no convolution state), equal sizes
    "ones": dict(vocab=97, width=64, streams=1, logit_softcap=30.0, norm={"eps": 1e-5}, layers=[
        latent(1, 32, 32, 32, 32, 0.2, ff=64), delta(1, 1, 32, 32, 1, ff=64), latent(1, 32, 32, 32, 32, 0.3, kv_from=0)]),
    # latent wide against the heads: prompts of some 90 tokens run expanded
    "wide": dict(vocab=320, width=192, streams=2, logit_softcap=20.0, norm={"eps": 1e-5}, layers=[
        latent(4, 32, 48, 64, 250, 0.18, ff=128), delta(4, 2, 64, 64, 4), latent(9, 16, 8, 24, 250, 0.3, kv_from=0, ff=700),
        latent(2, 100, 128, 48, 512, 0.1)]),
    # no delta layer: no recurrent state anywhere
    "attention": dict(vocab=128, width=96, streams=5, logit_softcap=8.0, norm={"eps": 1e-4}, layers=[
        latent(17, 8, 16, 24, 56, 0.4, ff=72), latent(3, 136, 144, 40, 130, 0.09)]),
    # only delta layers: nothing in the page cache
    "recurrent": dict(vocab=111, width=72, streams=4, logit_softcap=15.0, norm={"eps": 1e-5}, layers=[
        delta(2, 1, 130, 70, 5, ff=40), delta(4, 4, 8, 33, 4, ff=56)]),
}


def config(name: str) -> RuruzenConfig:
    return RuruzenConfig.from_dict({"architecture": "Ruruzen", **MODELS[name]})


def weights(cfg: RuruzenConfig, seed: int = 0, gate_rank: int | None = 12) -> dict:
    """Random weights with spread-out attention scores: the query up-projections are
    scaled so that far keys matter, and decays reach from fast to nearly none."""
    w = random_weights(cfg, seed, gate_rank=gate_rank)
    g = torch.Generator().manual_seed(seed + 1)
    for name in w:
        if name.endswith("mix.uq"):
            w[name] = (w[name].float() * 3).to(torch.bfloat16)
        if name.endswith("dt_bias"):
            w[name] = (torch.randn(w[name].shape, generator=g) * 2 - 3).to(torch.bfloat16)
    return w


_CACHE: dict = {}


def oracle_logits(name: str, tokens, seed: int = 0) -> torch.Tensor:
    """float64 logits of every position (prefixes of longer runs are reused)."""
    from oracles import ruruzen as O

    key = (name, seed)
    if key not in _CACHE:
        cfg = config(name)
        _CACHE[key] = (cfg.raw, {k: v.double() for k, v in weights(cfg, seed).items()}, {})
    raw, w, runs = _CACHE[key]
    tokens = tuple(int(t) for t in tokens)
    for done, logits in runs.items():
        if done[:len(tokens)] == tokens:
            return logits[:len(tokens)]
    with torch.no_grad():
        runs[tokens] = O.forward(raw, w, list(tokens))
    return runs[tokens]
