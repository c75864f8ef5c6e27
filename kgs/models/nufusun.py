"""Nufusun: configuration, tensor names and weights.

A decoder of parallel layers (one norm, attention and feed-forward both read its
output, both are added to the residual). Attention has no rotation: positions
enter as a learned bias per distance bucket; every head's scores are a learned
mixture of all heads' scores (talking heads), the softmax has one more term of
score 0 in its denominator, and the projections have biases. The feed-forward is
a mixture of experts with clamped gates, routed by the sigmoid of a linear map,
whose weight scales an expert's input. :class:`kgs.serve.nufusun.NufusunModel`
serves it.

:class:`NufusunConfig` reads ``config.json`` (every size and constant that can
differ between models); the rows of the distance table come from its tensor.
"""
from __future__ import annotations

import json
import math
from dataclasses import dataclass, field
from pathlib import Path

import torch

from .ruruzen import _positive

ARCHITECTURE = "Nufusun"
ATTENTION = "attention"


@dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int                     # query / key size of a head
    vdim: int                    # value size of a head
    scale: float
    bias_max: float              # distance from which the last bucket is used


@dataclass(frozen=True)
class ExpertsSpec:
    experts: int
    top: int
    ff: int
    limit: float


@dataclass(frozen=True)
class LayerSpec:
    mixer: AttentionSpec
    mlp: ExpertsSpec | None      # None: the layer has no feed-forward


def _number(where: str, d: dict, name: str) -> float:
    v = d.get(name)
    if not isinstance(v, (int, float)) or isinstance(v, bool) or not math.isfinite(v):
        raise ValueError(f"{where}: {name} must be a number, got {v!r}")
    return float(v)


def _layer(i: int, d: dict) -> LayerSpec:
    where, m = f"layer {i}", d.get("mixer")
    if d.get("type") != ATTENTION:
        raise ValueError(f"{where}: unknown mixer type {d.get('type')!r}")
    if not isinstance(m, dict):
        raise ValueError(f"{where}: no mixer")
    spec = AttentionSpec(*_positive(where, m, "heads", "kv_heads", "dim", "vdim"), _number(where, m, "scale"),
                         _number(where, m, "bias_max"))
    if spec.heads % spec.kv_heads:
        raise ValueError(f"{where}: heads {spec.heads} is not a multiple of kv_heads {spec.kv_heads}")
    mlp = d.get("mlp")
    if mlp is None:
        return LayerSpec(spec, None)
    if mlp.get("kind") != "moe":
        raise ValueError(f"{where}: unknown feed-forward kind {mlp.get('kind')!r}")
    n, top = _positive(where, mlp["router"], "experts", "top")
    if top > n:
        raise ValueError(f"{where}: top {top} of {n} experts")
    return LayerSpec(spec, ExpertsSpec(n, top, _positive(where, mlp["expert"], "ff")[0],
                                       _number(where, mlp["expert"], "limit")))


@dataclass(frozen=True)
class NufusunConfig:
    vocab: int
    width: int
    eps: float
    embed_scale: float
    layers: tuple[LayerSpec, ...]
    path: str | None = None      # folder with model.safetensors; None: random weights
    raw: dict = field(default_factory=dict, compare=False, repr=False)

    @classmethod
    def from_dict(cls, d: dict, path: str | None = None) -> "NufusunConfig":
        if d.get("architecture") != ARCHITECTURE:
            raise ValueError(f"architecture {d.get('architecture')!r} is not {ARCHITECTURE}")
        layers = tuple(_layer(i, entry) for i, entry in enumerate(d["layers"]))
        if not layers:
            raise ValueError("a model needs at least one layer")
        vocab, width = _positive("config", d, "vocab", "width")
        return cls(vocab, width, _number("norm", d["norm"], "eps"), _number("embedding", d["embedding"], "scale"),
                   layers, path, d)

    @classmethod
    def from_folder(cls, path) -> "NufusunConfig":
        return cls.from_dict(json.loads((Path(path) / "config.json").read_text()), str(path))

    # what a worker process needs to rebuild the configuration
    def spec(self) -> dict:
        return {"config": self.raw, "path": self.path}

    @classmethod
    def from_spec(cls, spec: dict) -> "NufusunConfig":
        return cls.from_dict(spec["config"], spec["path"])

    def load_weights(self, seed: int = 0, device="cpu") -> dict[str, torch.Tensor]:
        """The checkpoint's tensors by name, checked against the configuration,
        or random ones of the same shapes when there is no checkpoint."""
        if self.path is None:
            return random_weights(self, seed, device)
        from kgs.utils.safetensors import load_file

        w = load_file(Path(self.path) / "model.safetensors")
        check_weights(self, w)
        return w


def tensor_shapes(cfg: NufusunConfig, buckets: int = 32) -> dict[str, tuple]:
    """Every tensor of a model. ``buckets``: rows of the distance tables."""
    D = cfg.width
    s: dict[str, tuple] = {"embed": (cfg.vocab, D), "final.norm": (D,), "head": (cfg.vocab, D)}
    for i, layer in enumerate(cfg.layers):
        p, m, f = f"l{i}.", layer.mixer, layer.mlp
        s[p + "norm1"] = (D,)
        x = p + "mix."
        for n, c in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)):
            s |= {x + n: (c, D), f"{x}{n}.b": (c,)}
        s |= {x + "o": (D, m.heads * m.vdim), x + "o.b": (D,), x + "rel": (buckets, m.heads),
              x + "talk": (m.heads, m.heads), x + "temp": (m.heads,)}
        if f is not None:
            x = p + "mlp."
            s[x + "router"] = (f.experts, D)
            for e in range(f.experts):
                s |= {f"{x}e{e}.gate": (f.ff, D), f"{x}e{e}.up": (f.ff, D), f"{x}e{e}.down": (D, f.ff)}
    return s


def check_weights(cfg: NufusunConfig, w: dict[str, torch.Tensor]) -> None:
    """Names and shapes against the configuration (the distance tables' rows are free)."""
    want = tensor_shapes(cfg)
    missing = sorted(set(want) - set(w))
    if missing:
        raise ValueError(f"checkpoint lacks {len(missing)} tensors, first {missing[:4]}")
    for name, shape in want.items():
        got = tuple(w[name].shape)
        ok = len(got) == 2 and got[0] >= 2 and got[1] == shape[1] if name.endswith(".rel") else got == shape
        if not ok:
            raise ValueError(f"tensor {name} has shape {got}, expected {shape}")
    for i, layer in enumerate(cfg.layers):
        rows = w[f"l{i}.mix.rel"].shape[0]
        if layer.mixer.bias_max <= rows // 2:
            raise ValueError(f"layer {i}: bias_max {layer.mixer.bias_max} is not above half its {rows} distance buckets")


def random_weights(cfg: NufusunConfig, seed: int = 0, device="cpu", buckets: int = 32) -> dict[str, torch.Tensor]:
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, buckets).items():
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g, device=device)
        if leaf in ("norm", "norm1"):
            t = 0.1 * r
        elif leaf == "b":
            t = 0.1 * r
        elif leaf == "temp":
            t = 1 + 0.1 * r
        elif leaf == "talk":
            t = torch.eye(shape[0], device=device) + 0.3 * r * shape[0] ** -0.5
        elif leaf in ("embed", "rel"):
            t = r
        else:
            t = r * shape[-1] ** -0.5
        out[name] = t.to(torch.bfloat16)
    return out
