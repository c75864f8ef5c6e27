"""Nokipel: configuration, tensor names and weights.

A decoder whose layers mix tokens either with chunked attention (grouped key heads,
biased projections, rotary positions on neighbouring pairs, keys of the query's own chunk
of positions only) or with lightning attention (a linear recurrence with a fixed decay
per head); feed-forwards are dense with a clamped gate or a group-limited mixture of
experts with identity experts and a gated shared expert. Norms work on equal parts of the
row. A run of layers can be passed several times with the same weights; every later pass
starts with the embedding output added. :class:`kgs.serve.nokipel.NokipelModel` serves it.

:class:`NokipelConfig` reads ``config.json`` (every size and constant that can differ
between models).
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from pathlib import Path

import torch

from .nufusun import _number
from .ruruzen import _positive

ARCHITECTURE = "Nokipel"
ATTENTION, LIGHTNING = "attention", "lightning"


@dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int                     # query / key size of a head
    vdim: int                    # value size of a head
    scale: float
    chunk: int                   # positions of a chunk, 0: every earlier key is visible
    rot_dims: int                # rotated dimensions of a head
    rot_base: float


@dataclass(frozen=True)
class LightningSpec:
    heads: int
    dim: int
    vdim: int
    decay: tuple[float, ...]     # per head


@dataclass(frozen=True)
class DenseSpec:
    ff: int
    limit: float


@dataclass(frozen=True)
class ExpertsSpec:
    experts: int
    identity: int                # outputs that return their input
    top: int
    groups: int
    keep: int                    # groups whose experts can be chosen
    scale: float
    ff: int
    shared_ff: int               # 0: no shared expert


@dataclass(frozen=True)
class LayerSpec:
    mixer: AttentionSpec | LightningSpec
    mlp: DenseSpec | ExpertsSpec | None  # None: the layer has no feed-forward


def _mixer(where: str, kind: str, m) -> AttentionSpec | LightningSpec:
    if not isinstance(m, dict):
        raise ValueError(f"{where}: no mixer")
    if kind == ATTENTION:
        heads, kv = _positive(where, m, "heads", "kv_heads")
        if heads % kv:
            raise ValueError(f"{where}: heads {heads} is not a multiple of kv_heads {kv}")
        dim, vdim = _positive(where, m, "dim", "vdim")
        scale, rot = _number(where, m, "scale"), m.get("rot") or {}
        dims = rot.get("dims", 0)
        if not isinstance(dims, int) or dims < 0 or dims % 2 or dims > dim:
            raise ValueError(f"{where}: rot.dims {dims!r} is no even number up to {dim}")
        base = _number(where, rot, "base") if dims else 1.0
        chunk = _positive(where, m["mask"], "size")[0] if m.get("mask") else 0
        if scale <= 0 or base <= 0:
            raise ValueError(f"{where}: scale {scale} and rot.base {base} must be positive")
        return AttentionSpec(heads, kv, dim, vdim, scale, chunk, dims, base)
    if kind == LIGHTNING:
        heads, dim, vdim = _positive(where, m, "heads", "dim", "vdim")
        decay = m.get("decay")
        if not isinstance(decay, (list, tuple)) or len(decay) != heads:
            raise ValueError(f"{where}: decay must give one number for each of the {heads} heads")
        return LightningSpec(heads, dim, vdim, tuple(_number(where, {"decay": d}, "decay") for d in decay))
    raise ValueError(f"{where}: unknown mixer type {kind!r}")


def _mlp(where: str, d) -> DenseSpec | ExpertsSpec | None:
    if d is None:
        return None
    if d.get("kind") == "dense":
        return DenseSpec(_positive(where, d, "ff")[0], _number(where, d, "limit"))
    if d.get("kind") != "moe":
        raise ValueError(f"{where}: unknown feed-forward kind {d.get('kind')!r}")
    r = d["router"]
    n, top = _positive(where, r, "experts", "top")
    identity = r.get("identity") or 0
    if not isinstance(identity, int) or identity < 0:
        raise ValueError(f"{where}: identity must be a number of experts, got {identity!r}")
    groups, keep = _positive(where, r["groups"], "count", "keep") if r.get("groups") else (1, 1)
    if (n + identity) % groups or keep > groups or top > (n + identity) // groups * keep:
        raise ValueError(f"{where}: cannot choose {top} of {n + identity} experts in {keep} of {groups} groups")
    scale = _number(where, r, "scale") if "scale" in r else 1.0
    shared = _positive(where, d["shared"], "ff")[0] if d.get("shared") else 0
    return ExpertsSpec(n, identity, top, groups, keep, scale, _positive(where, d["expert"], "ff")[0], shared)


@dataclass(frozen=True)
class NokipelConfig:
    vocab: int
    width: int
    eps: float
    norm_groups: int
    embed_scale: float
    layers: tuple[LayerSpec, ...]
    loop: tuple[int, int, int]   # layers start .. stop - 1 run this many times
    path: str | None = None      # folder with model.safetensors; None: random weights
    raw: dict = field(default_factory=dict, compare=False, repr=False)

    @classmethod
    def from_dict(cls, d: dict, path: str | None = None) -> "NokipelConfig":
        if d.get("architecture") != ARCHITECTURE:
            raise ValueError(f"architecture {d.get('architecture')!r} is not {ARCHITECTURE}")
        layers = tuple(LayerSpec(_mixer(f"layer {i}", e.get("type"), e.get("mixer")), _mlp(f"layer {i}", e.get("mlp")))
                       for i, e in enumerate(d["layers"]))
        if not layers:
            raise ValueError("a model needs at least one layer")
        vocab, width = _positive("config", d, "vocab", "width")
        norm = d["norm"]
        groups = _positive("norm", norm, "groups")[0] if "groups" in norm else 1
        if width % groups:
            raise ValueError(f"width {width} has no {groups} equal parts")
        loop = (0, 0, 1)
        if d.get("loop"):
            lp = d["loop"]
            start, (stop, times) = lp.get("start"), _positive("loop", lp, "stop", "times")
            if not isinstance(start, int) or not 0 <= start < stop <= len(layers):
                raise ValueError(f"loop over layers {start!r} .. {stop} of {len(layers)}")
            loop = (start, stop, times)
        return cls(vocab, width, _number("norm", norm, "eps"), groups, _number("embedding", d["embedding"], "scale"),
                   layers, loop, path, d)

    @classmethod
    def from_folder(cls, path) -> "NokipelConfig":
        return cls.from_dict(json.loads((Path(path) / "config.json").read_text()), str(path))

    # what a worker process needs to rebuild the configuration
    def spec(self) -> dict:
        return {"config": self.raw, "path": self.path}

    @classmethod
    def from_spec(cls, spec: dict) -> "NokipelConfig":
        return cls.from_dict(spec["config"], spec["path"])

    @property
    def runs(self) -> list[tuple[int, bool]]:
        """Every layer run in order: the layer, and whether the embedding output is added
        before it."""
        start, stop, times = self.loop
        out = [(i, False) for i in range(start)]
        for t in range(times):
            out += [(i, t > 0 and i == start) for i in range(start, stop)]
        return out + [(i, False) for i in range(stop, len(self.layers))]

    @property
    def has_state(self) -> bool:
        return any(isinstance(x.mixer, LightningSpec) for x in self.layers)

    def load_weights(self, seed: int = 0, device="cpu") -> dict[str, torch.Tensor]:
        """The checkpoint's tensors by name, checked against the configuration,
        or random ones of the same shapes when there is no checkpoint."""
        if self.path is None:
            return random_weights(self, seed, device)
        from kgs.utils.safetensors import load_file

        w = load_file(Path(self.path) / "model.safetensors")
        check_weights(self, w)
        return w


def tensor_shapes(cfg: NokipelConfig) -> dict[str, tuple]:
    """Every tensor of a model."""
    D = cfg.width
    s: dict[str, tuple] = {"embed": (cfg.vocab, D), "final.norm": (D,), "head": (cfg.vocab, D)}

    def gated(p, ff):
        return {p + "gate": (ff, D), p + "up": (ff, D), p + "down": (D, ff)}

    for i, layer in enumerate(cfg.layers):
        p, m, f = f"l{i}.", layer.mixer, layer.mlp
        s[p + "norm1"] = (D,)
        x = p + "mix."
        if isinstance(m, AttentionSpec):
            for n, c in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)):
                s |= {x + n: (c, D), f"{x}{n}.b": (c,)}
        else:
            hk, hv = m.heads * m.dim, m.heads * m.vdim
            s |= {x + "q": (hk, D), x + "k": (hk, D), x + "v": (hv, D), x + "g": (hv, D), x + "norm": (hv,)}
        s[x + "o"] = (D, m.heads * m.vdim)
        if f is None:
            continue
        s[p + "norm2"] = (D,)
        x = p + "mlp."
        if isinstance(f, DenseSpec):
            s |= gated(x, f.ff)
            continue
        s |= {x + "router": (f.experts + f.identity, D), x + "correction": (f.experts + f.identity,)}
        for e in range(f.experts):
            s |= gated(f"{x}e{e}.", f.ff)
        if f.shared_ff:
            s |= gated(x + "shared.", f.shared_ff) | {x + "shared.sg": (1, D)}
    return s


def check_weights(cfg: NokipelConfig, w: dict[str, torch.Tensor]) -> None:
    """Names and shapes against the configuration."""
    want = tensor_shapes(cfg)
    missing = sorted(set(want) - set(w))
    if missing:
        raise ValueError(f"checkpoint lacks {len(missing)} tensors, first {missing[:4]}")
    for name, shape in want.items():
        if tuple(w[name].shape) != shape:
            raise ValueError(f"tensor {name} has shape {tuple(w[name].shape)}, expected {shape}")


def random_weights(cfg: NokipelConfig, seed: int = 0, device="cpu") -> dict[str, torch.Tensor]:
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g, device=device)
        if leaf in ("norm", "norm1", "norm2"):
            t = 1 + 0.1 * r
        elif leaf == "b":
            t = 0.1 * r
        elif leaf == "correction":
            t = 0.05 * r
        elif leaf == "embed":
            t = r
        else:
            t = r * shape[-1] ** -0.5
        out[name] = t.to(torch.bfloat16)
    return out
