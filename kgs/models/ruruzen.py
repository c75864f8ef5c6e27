"""Ruruzen: configuration, tensor names and weights.

A decoder whose residual is several parallel streams (hyper-connections) and
whose layers mix tokens either with latent attention (no positions, one cached
latent vector per token, which later layers may share) or with a gated delta rule
that decays every key channel by itself; dense tanh-gelu feed-forwards, tied
embedding and output, soft-capped logits. :class:`kgs.serve.hybrid.HybridModel`
serves it.

:class:`RuruzenConfig` reads ``config.json`` (every size and constant that can
differ between models); the ranks of the delta mixer's two low-rank gates are
not in it and come from the tensors' shapes.
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from pathlib import Path

import torch

ARCHITECTURE = "Ruruzen"
LATENT, DELTA = "latent_attention", "channel_delta"


def _positive(where: str, d: dict, *names: str) -> list[int]:
    out = []
    for n in names:
        v = d.get(n)
        if not isinstance(v, int) or isinstance(v, bool) or v <= 0:
            raise ValueError(f"{where}: {n} must be a positive integer, got {v!r}")
        out.append(v)
    return out


@dataclass(frozen=True)
class LatentSpec:
    heads: int
    dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    kv_from: int | None = None   # the layer whose cached latent this one reads (None: its own)
    rot_dim: int = 0             # further query / key dimensions of a head that turn with the position
    rot_base: float = 1.0
    window: int = 0              # keys a token sees, itself among them; 0: all
    gate_each: bool = False      # the output gate has a number per element, not per head


@dataclass(frozen=True)
class DeltaSpec:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int                    # taps of the short convolutions


@dataclass(frozen=True)
class LayerSpec:
    mixer: LatentSpec | DeltaSpec
    ff: int | None               # feed-forward width, None: the layer has no feed-forward

    @property
    def type(self) -> str:
        return LATENT if isinstance(self.mixer, LatentSpec) else DELTA


def _layer(i: int, d: dict, earlier: list[LayerSpec]) -> LayerSpec:
    where, m = f"layer {i}", d.get("mixer")
    if not isinstance(m, dict):
        raise ValueError(f"{where}: no mixer")
    if d["type"] == LATENT:
        src = m.get("kv_from")
        if src == i:
            src = None
        spec = LatentSpec(*_positive(where, m, "heads", "dim", "vdim", "q_rank", "kv_rank"), float(m["scale"]), src)
        if src is not None:
            owner = earlier[src].mixer if isinstance(src, int) and 0 <= src < i else None
            if not isinstance(owner, LatentSpec) or owner.kv_from is not None or owner.kv_rank != spec.kv_rank:
                raise ValueError(f"{where}: kv_from {src!r} is no earlier layer with its own latent of size "
                                 f"{spec.kv_rank}")
    elif d["type"] == DELTA:
        spec = DeltaSpec(*_positive(where, m, "heads", "kv_heads", "dim", "vdim", "conv"))
        if spec.heads % spec.kv_heads:
            raise ValueError(f"{where}: heads {spec.heads} is not a multiple of kv_heads {spec.kv_heads}")
    else:
        raise ValueError(f"{where}: unknown mixer type {d['type']!r}")
    mlp = d.get("mlp")
    if mlp is not None and mlp.get("kind") != "dense":
        raise ValueError(f"{where}: unknown feed-forward kind {mlp.get('kind')!r}")
    return LayerSpec(spec, None if mlp is None else _positive(where, mlp, "ff")[0])


@dataclass(frozen=True)
class RuruzenConfig:
    vocab: int
    width: int
    streams: int
    eps: float
    logit_softcap: float
    layers: tuple[LayerSpec, ...]
    path: str | None = None      # folder with model.safetensors; None: random weights
    raw: dict = field(default_factory=dict, compare=False, repr=False)

    @classmethod
    def from_dict(cls, d: dict, path: str | None = None) -> "RuruzenConfig":
        if d.get("architecture") != ARCHITECTURE:
            raise ValueError(f"architecture {d.get('architecture')!r} is not {ARCHITECTURE}")
        layers: list[LayerSpec] = []
        for i, entry in enumerate(d["layers"]):
            layers.append(_layer(i, entry, layers))
        if not layers:
            raise ValueError("a model needs at least one layer")
        vocab, width, streams = _positive("config", d, "vocab", "width", "streams")
        return cls(vocab, width, streams, float(d["norm"]["eps"]), float(d.get("logit_softcap") or 0.0),
                   tuple(layers), path, d)

    @classmethod
    def from_folder(cls, path) -> "RuruzenConfig":
        return cls.from_dict(json.loads((Path(path) / "config.json").read_text()), str(path))

    # what a worker process needs to rebuild the configuration
    def spec(self) -> dict:
        return {"config": self.raw, "path": self.path}

    @classmethod
    def from_spec(cls, spec: dict) -> "RuruzenConfig":
        return cls.from_dict(spec["config"], spec["path"])

    @property
    def has_state(self) -> bool:
        return any(isinstance(x.mixer, DeltaSpec) for x in self.layers)

    def load_weights(self, seed: int = 0, device="cpu") -> dict[str, torch.Tensor]:
        """The checkpoint's tensors by name, checked against the configuration,
        or random ones of the same shapes when there is no checkpoint."""
        if self.path is None:
            return random_weights(self, seed, device)
        from kgs.utils.safetensors import load_file

        w = load_file(Path(self.path) / "model.safetensors")
        check_weights(self, w)
        return w


def tensor_shapes(cfg: RuruzenConfig, gate_rank: int | None = None) -> dict[str, tuple]:
    """Every tensor of a model. ``gate_rank``: rank of the delta mixers' low-rank
    decay and output gates (default: the mixer's key size)."""
    D = cfg.width
    s: dict[str, tuple] = {"embed": (cfg.vocab, D), "embed.norm": (D,), "final.norm": (D,)}
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}.", layer.mixer
        for q in (1, 2) if layer.ff is not None else (1,):
            s |= {f"{p}norm{q}": (D,), f"{p}hc{q}.in": (cfg.streams,), f"{p}hc{q}.out": (cfg.streams,),
                  f"{p}hc{q}.mix": (cfg.streams, cfg.streams)}
        x = p + "mix."
        if isinstance(m, LatentSpec):
            s |= {x + "dq": (m.q_rank, D), x + "dq.norm": (m.q_rank,), x + "uq": (m.heads * m.dim, m.q_rank),
                  x + "uk": (m.heads * m.dim, m.kv_rank), x + "uv": (m.heads * m.vdim, m.kv_rank),
                  x + "g": (m.heads, D), x + "o": (D, m.heads * m.vdim)}
            if m.kv_from is None:
                s |= {x + "dkv": (m.kv_rank, D), x + "dkv.norm": (m.kv_rank,)}
        else:
            gk, hv, r = m.kv_heads * m.dim, m.heads * m.vdim, gate_rank or m.dim
            for n, c in (("q", gk), ("k", gk), ("v", hv)):
                s |= {x + n: (c, D), f"{x}{n}.conv": (c, m.conv)}
            s |= {x + "b": (m.heads, D), x + "A_log": (m.heads,), x + "dt_bias": (m.heads * m.dim,),
                  x + "a1": (r, D), x + "a2": (m.heads * m.dim, r), x + "g1": (r, D), x + "g2": (hv, r),
                  x + "norm": (m.vdim,), x + "o": (D, hv)}
        if layer.ff is not None:
            s |= {p + "mlp.gate": (layer.ff, D), p + "mlp.up": (layer.ff, D), p + "mlp.down": (D, layer.ff)}
    return s


def check_weights(cfg: RuruzenConfig, w: dict[str, torch.Tensor]) -> None:
    """Names and shapes against the configuration (the low-rank gates' ranks are free)."""
    want = tensor_shapes(cfg)
    missing = sorted(set(want) - set(w))
    if missing:
        raise ValueError(f"checkpoint lacks {len(missing)} tensors, first {missing[:4]}")
    for name, shape in want.items():
        got, free = tuple(w[name].shape), name.rsplit(".", 1)[-1]
        if free in ("a1", "g1"):
            ok = len(got) == 2 and got[1] == shape[1]
        elif free in ("a2", "g2"):
            rank = w[name[:-1] + "1"].shape[0]
            ok = got == (shape[0], rank)
        else:
            ok = got == shape
        if not ok:
            raise ValueError(f"tensor {name} has shape {got}, expected {shape}")


def random_weights(cfg: RuruzenConfig, seed: int = 0, device="cpu", gate_rank: int | None = None
                   ) -> dict[str, torch.Tensor]:
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg, gate_rank).items():
        leaf = name.rsplit(".", 1)[-1]
        r = torch.randn(shape, generator=g, device=device)
        if leaf in ("norm", "norm1", "norm2"):
            t = 1 + 0.1 * r
        elif leaf == "in":
            t = 1.0 / cfg.streams + 0.1 * r
        elif leaf == "out":
            t = 1 + 0.1 * r
        elif leaf == "mix":
            t = torch.eye(cfg.streams, device=device) + 0.05 * r
        elif leaf == "A_log":
            t = 0.5 * r - 1
        elif leaf == "dt_bias":
            t = r - 2
        elif name == "embed":
            t = r
        else:
            t = r * shape[-1] ** -0.5
        out[name] = t.to(torch.bfloat16)
    return out
