"""Vumalix: configuration, tensor names and weights.

A decoder that norms what its sublayers put out (by one number per norm) and lets them
read the residual itself; in front of every mixer a short causal convolution adds
neighbouring positions on each channel. Layers mix tokens with latent attention (a cached
latent, a rotated key part shared by the heads, a sliding window, an output gate per
element) or with differential attention (two softmaxes per head over the same values,
normed queries and keys, no positions but a query temperature that grows with them).
Feed-forwards are ungated: a sum of normed powers. A layer can use another layer's
weights with a cache and state of its own. :class:`kgs.serve.vumalix.VumalixModel` serves it.

:class:`VumalixConfig` reads ``config.json`` (every size and constant that can differ
between models).
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from pathlib import Path

import torch

from .nufusun import _number
from .ruruzen import LatentSpec, _positive

ARCHITECTURE = "Vumalix"
LATENT, ATTENTION = "latent_attention", "attention"


@dataclass(frozen=True)
class DiffAttentionSpec:
    heads: int
    kv_heads: int
    dim: int                     # query / key size of one map of a head
    vdim: int                    # value size of a head
    scale: float
    diff: float                  # what lambda starts from
    temp_coef: float             # queries times 1 + coef ln(floor((p + 1) / every) + 1)
    temp_every: int


@dataclass(frozen=True)
class LayerSpec:
    mixer: LatentSpec | DiffAttentionSpec
    ff: int | None               # None: the layer has no feed-forward
    owner: int                   # the layer whose weights it uses


def _mixer(where: str, kind: str, m) -> LatentSpec | DiffAttentionSpec:
    if not isinstance(m, dict):
        raise ValueError(f"{where}: no mixer")
    scale = _number(where, m, "scale")
    if scale <= 0:
        raise ValueError(f"{where}: scale {scale} must be positive")
    if kind == LATENT:
        heads, dim, vdim, qr, kr, rot = _positive(where, m, "heads", "dim", "vdim", "q_rank", "kv_rank", "rot_dim")
        dims, base = _positive(where, m["rot"], "dims")[0], _number(where, m["rot"], "base")
        if dims != rot or rot % 2 or base <= 0:
            raise ValueError(f"{where}: rot.dims {dims} must be the even rot_dim {rot}, rot.base {base} positive")
        window = _positive(where, m["mask"], "size")[0] if m.get("mask") else 0
        return LatentSpec(heads, dim, vdim, qr, kr, scale, rot_dim=rot, rot_base=base, window=window, gate_each=True)
    if kind == ATTENTION:
        heads, kv, dim, vdim = _positive(where, m, "heads", "kv_heads", "dim", "vdim")
        if heads % kv:
            raise ValueError(f"{where}: heads {heads} is not a multiple of kv_heads {kv}")
        t = m["q_temp"]
        return DiffAttentionSpec(heads, kv, dim, vdim, scale, _number(where, m, "diff"), _number(where, t, "coef"),
                                 _positive(where, t, "every")[0])
    raise ValueError(f"{where}: unknown mixer type {kind!r}")


def _owner(entries, i: int) -> int:
    """The layer whose weights layer ``i`` uses."""
    j = i
    for _ in entries:
        k = entries[j].get("weights_of")
        if k is None or k == j:
            return j
        if not isinstance(k, int) or isinstance(k, bool) or not 0 <= k < len(entries):
            raise ValueError(f"layer {j}: weights_of {k!r} is no layer")
        j = k
    raise ValueError(f"layer {i}: no layer has the weights")


def _layers(entries) -> tuple[LayerSpec, ...]:
    out = []
    for i, e in enumerate(entries):
        where, f = f"layer {i}", e.get("mlp")
        if f is not None and f.get("kind") != "dense":
            raise ValueError(f"{where}: unknown feed-forward kind {f.get('kind')!r}")
        out.append(LayerSpec(_mixer(where, e.get("type"), e.get("mixer")), None if f is None else _positive(where, f, "ff")[0],
                             _owner(entries, i)))
    if not out:
        raise ValueError("a model needs at least one layer")
    for i, x in enumerate(out):
        o = out[x.owner]
        if (o.mixer, o.ff) != (x.mixer, x.ff):
            raise ValueError(f"layer {i} cannot use the weights of layer {x.owner}, which has other sizes")
    return tuple(out)


@dataclass(frozen=True)
class VumalixConfig:
    vocab: int
    width: int
    eps: float
    taps: int                    # of the convolution in front of every mixer
    layers: tuple[LayerSpec, ...]
    path: str | None = None      # folder with model.safetensors; None: random weights
    raw: dict = field(default_factory=dict, compare=False, repr=False)

    @classmethod
    def from_dict(cls, d: dict, path: str | None = None) -> "VumalixConfig":
        if d.get("architecture") != ARCHITECTURE:
            raise ValueError(f"architecture {d.get('architecture')!r} is not {ARCHITECTURE}")
        vocab, width = _positive("config", d, "vocab", "width")
        return cls(vocab, width, _number("norm", d["norm"], "eps"), _positive("canon", d["canon"], "taps")[0],
                   _layers(d["layers"]), path, d)

    @classmethod
    def from_folder(cls, path) -> "VumalixConfig":
        return cls.from_dict(json.loads((Path(path) / "config.json").read_text()), str(path))

    # what a worker process needs to rebuild the configuration
    def spec(self) -> dict:
        return {"config": self.raw, "path": self.path}

    @classmethod
    def from_spec(cls, spec: dict) -> "VumalixConfig":
        return cls.from_dict(spec["config"], spec["path"])

    @property
    def owners(self) -> list[int]:
        """The layers with weights of their own."""
        return sorted({x.owner for x in self.layers})

    @property
    def has_state(self) -> bool:
        return self.taps > 1

    def load_weights(self, seed: int = 0, device="cpu") -> dict[str, torch.Tensor]:
        """The checkpoint's tensors by name, checked against the configuration,
        or random ones of the same shapes when there is no checkpoint."""
        if self.path is None:
            return random_weights(self, seed, device)
        from kgs.utils.safetensors import load_file

        w = load_file(Path(self.path) / "model.safetensors")
        check_weights(self, w)
        return w


def tensor_shapes(cfg: VumalixConfig) -> dict[str, tuple]:
    """Every tensor of a model."""
    D = cfg.width
    s: dict[str, tuple] = {"embed": (cfg.vocab, D), "final.norm": (), "head": (cfg.vocab, D)}
    for i in cfg.owners:
        p, m, ff = f"l{i}.", cfg.layers[i].mixer, cfg.layers[i].ff
        x, hv = p + "mix.", m.heads * m.vdim
        s |= {p + "norm1": (), p + "canon1": (D, cfg.taps), x + "o": (D, hv)}
        if isinstance(m, LatentSpec):
            s |= {x + "dq": (m.q_rank, D), x + "dq.norm": (m.q_rank,), x + "uq": (m.heads * (m.dim + m.rot_dim), m.q_rank),
                  x + "dkv": (m.kv_rank + m.rot_dim, D), x + "dkv.norm": (m.kv_rank,),
                  x + "uk": (m.heads * m.dim, m.kv_rank), x + "uv": (hv, m.kv_rank), x + "g": (hv, D)}
        else:
            s |= {x + "q": (m.heads * 2 * m.dim, D), x + "k": (m.kv_heads * 2 * m.dim, D), x + "v": (m.kv_heads * m.vdim, D)}
            s |= {x + n: (m.dim,) for n in ("q.norm", "k.norm", "lq1", "lk1", "lq2", "lk2")}
        if ff is not None:
            s |= {p + "norm2": (), p + "mlp.up": (ff, D), p + "mlp.down": (D, ff), p + "mlp.act": (4,)}
    return s


def check_weights(cfg: VumalixConfig, w: dict[str, torch.Tensor]) -> None:
    """Names and shapes against the configuration."""
    want = tensor_shapes(cfg)
    missing = sorted(set(want) - set(w))
    if missing:
        raise ValueError(f"checkpoint lacks {len(missing)} tensors, first {missing[:4]}")
    for name, shape in want.items():
        if tuple(w[name].shape) != shape:
            raise ValueError(f"tensor {name} has shape {tuple(w[name].shape)}, expected {shape}")


def random_weights(cfg: VumalixConfig, seed: int = 0, device="cpu") -> dict[str, torch.Tensor]:
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g, device=device)
        if leaf in ("norm", "norm1", "norm2"):
            t = 1 + 0.1 * r
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            t = 0.5 * r * shape[0] ** -0.5
        elif leaf == "canon1":
            t = 0.3 * r
        elif leaf == "act":
            t = torch.tensor([0.8, 0.6, 0.4, 0.1], device=device) + 0.1 * r
        elif leaf == "embed":
            t = r
        else:
            t = r * shape[-1] ** -0.5
        out[name] = t.to(torch.bfloat16)
    return out
