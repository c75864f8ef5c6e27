"""Small Nufusun configurations and weights for the tests, and runs of the oracle on
them. Together they cover every kernel form: one to eight slots of heads, groups that
are no multiple of four or straddle MFMA tiles, more slots or larger heads than the
tiled or the MFMA kernels take, one expert, all experts, more than the MFMA router's."""
import torch

from kgs.models.nufusun import NufusunConfig, random_weights


def layer(heads, kv_heads, dim, vdim, scale, bias_max, moe=None):
    """``moe``: (experts, top, ff, limit) or None."""
    mlp = None
    if moe is not None:
        e, top, ff, limit = moe
        mlp = {"kind": "moe", "router": {"experts": e, "top": top}, "expert": {"ff": ff, "limit": limit}}
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": bias_max}}


MODELS = {
    # unlike layers, one without a feed-forward
    "mixed": (dict(vocab=203, width=140, embedding={"scale": 3.5}, norm={"eps": 3e-6}, layers=[
        layer(4, 2, 24, 40, 0.2, 20, (5, 2, 48, 0.7)), layer(5, 1, 80, 112, 0.11, 90.5),
        layer(8, 8, 64, 64, 0.125, 33, (7, 7, 130, 2.5)), layer(12, 3, 40, 20, 0.17, 50, (3, 1, 72, 1.5))]), 8),
    # 20 heads in groups of 5 (two head tiles, eight slots), wide heads beside narrow ones
    "groups": (dict(vocab=131, width=300, embedding={"scale": 1.0}, norm={"eps": 1e-5}, layers=[
        layer(20, 4, 100, 50, 0.1, 64, (20, 3, 96, 1.0)), layer(30, 5, 64, 128, 0.12, 128, (1, 1, 200, 0.4)),
        layer(32, 8, 128, 128, 0.09, 200, (130, 4, 24, 1.2))]), 32),
    # one head; only rows kernels: 18 key heads, 34 and 64 query heads; beyond MFMA: dim 160, 66 heads
    "rows": (dict(vocab=97, width=96, embedding={"scale": 2.0}, norm={"eps": 1e-4}, layers=[
        layer(1, 1, 16, 16, 0.3, 10, (4, 2, 40, 1.0)), layer(18, 18, 32, 24, 0.2, 40, (18, 2, 64, 3.0)),
        layer(34, 2, 48, 72, 0.15, 30), layer(64, 16, 16, 128, 0.25, 100), layer(3, 1, 160, 32, 0.08, 17, (40, 5, 16, 0.9)),
        layer(66, 6, 20, 28, 0.2, 21)]), 6),
}


def config(name: str) -> NufusunConfig:
    return NufusunConfig.from_dict({"architecture": "Nufusun", **MODELS[name][0]})


def weights(cfg: NufusunConfig, buckets: int, seed: int = 0) -> dict:
    """Random weights with spread-out scores: queries scaled so that far keys matter, and
    experts scaled down, so that in bf16 a choice between two that nearly tie matters less."""
    w = random_weights(cfg, seed, buckets=buckets)
    for name in w:
        if name.endswith("mix.q"):
            w[name] = (w[name].float() * 2).to(torch.bfloat16)
        elif name.endswith(".down"):
            w[name] = (w[name].float() * 0.3).to(torch.bfloat16)
        elif name.endswith(".b"):
            w[name] = (w[name].float() * 4).to(torch.bfloat16)
    return w


def model(name: str):
    cfg = config(name)
    return cfg, weights(cfg, MODELS[name][1])


_CACHE: dict = {}


def oracle_logits(name: str, tokens) -> torch.Tensor:
    """float64 logits of every position (prefixes of longer runs are reused)."""
    from oracles import nufusun as O

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
