"""Small Nokipel configurations and weights for the tests, and runs of the oracle on them.
Together they cover every branch: layers of each kind with and without a feed-forward, runs
of layers passed several times from the first layer, from inside and to the last one, norm
parts that are a multiple of eight columns or not, groups, identity and shared experts or
none of them, chunks shorter and longer than a page, and head sizes that the MFMA and the
chunked kernels take, pad or leave to the plain ones."""
import torch

from kgs.models.nokipel import NokipelConfig, random_weights


def attention(heads, kv_heads, dim, vdim, scale, chunk, rot, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                      "mask": {"size": chunk}, "rot": {"dims": rot[0], "base": rot[1]}}}


def lightning(dim, vdim, decay, mlp=None):
    return {"type": "lightning", "mlp": mlp, "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": decay}}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, identity=0, groups=None, scale=1.0, shared=None):
    r = {"experts": experts, "top": top, "identity": identity, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "router": r, "expert": {"ff": ff}, **({"shared": {"ff": shared}} if shared else {})}


MODELS = {
    "mixed": dict(vocab=203, width=140, embedding={"scale": 3.5}, norm={"eps": 3e-6, "groups": 5},
                  loop={"start": 1, "stop": 3, "times": 3}, layers=[
        lightning(24, 40, [0.5, 0.9, 0.98, 0.9995], dense(72, 0.8)),
        attention(4, 2, 24, 40, 0.3, 20, (12, 1e3), moe(5, 3, 48, identity=1, groups=(3, 2), scale=1.3, shared=56)),
        lightning(48, 16, [0.97, 0.6], moe(7, 3, 40)),
        attention(3, 1, 80, 112, 0.15, 50, (80, 1e4))]),
    "first": dict(vocab=131, width=192, embedding={"scale": 1.0}, norm={"eps": 1e-5, "groups": 4},
                  loop={"start": 0, "stop": 2, "times": 2}, layers=[
        attention(16, 1, 64, 64, 0.2, 33, (2, 10.0), moe(14, 4, 32, identity=2, groups=(4, 3), scale=2.5, shared=130)),
        lightning(64, 128, [0.9, 0.99, 0.3, 1.0, 0.0, 0.995], dense(200, 2.0))]),
    # no state: attention only, whole-row norm, no loop
    "stateless": dict(vocab=97, width=256, embedding={"scale": 2.0}, norm={"eps": 1e-4, "groups": 1}, layers=[
        attention(8, 4, 128, 128, 0.1, 64, (128, 5e5), dense(512, 1.0)),
        attention(20, 1, 48, 24, 0.2, 7, (20, 100.0), moe(3, 3, 130, shared=40)),
        attention(2, 2, 100, 64, 0.13, 1000, (50, 1e4), dense(96, 0.3))]),
    # beyond the MFMA and chunk kernels' sizes; a loop of the last layer
    "large": dict(vocab=150, width=320, embedding={"scale": 1.5}, norm={"eps": 1e-5, "groups": 8},
                  loop={"start": 3, "stop": 4, "times": 3}, layers=[
        attention(6, 3, 160, 48, 0.08, 45, (64, 1e5), moe(60, 2, 16, identity=4, groups=(8, 2), shared=24)),
        lightning(200, 136, [0.95, 0.999]),
        attention(66, 6, 20, 28, 0.2, 31, (20, 30.0), dense(40, 1.5)),
        lightning(128, 256, [0.7, 0.999, 0.98], dense(64, 1.0))]),
}


def config(name: str) -> NokipelConfig:
    return NokipelConfig.from_dict({"architecture": "Nokipel", **MODELS[name]})


def weights(cfg: NokipelConfig, seed: int = 0) -> dict:
    """Random weights with spread-out scores: queries scaled so that far keys matter, and
    experts scaled down, so that in bf16 a choice between two that nearly tie matters less."""
    w = random_weights(cfg, seed)
    for name in w:
        f = 2 if name.endswith("mix.q") else 4 if name.endswith(".b") else 0.3 if ".e" in name and name.endswith(".down") else 1
        w[name] = (w[name].float() * f).to(torch.bfloat16)
    return w


def model(name: str):
    cfg = config(name)
    return cfg, weights(cfg)


_CACHE: dict = {}


def oracle_logits(name: str, tokens) -> torch.Tensor:
    """float64 logits of every position (prefixes of longer runs are reused)."""
    from oracles import nokipel as O

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
