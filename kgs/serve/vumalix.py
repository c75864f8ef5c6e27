"""Serving model of layer stacks that mix windowed latent attention and differential attention
with normed-power feed-forwards, on a residual that norms its sublayers' outputs and
convolves their inputs over time (:mod:`kgs.models.vumalix`).

Every step is one ragged batch (:class:`kgs.serve.ragged.Batch`). A sublayer is ``h ->
mixer or feed-forward -> y`` between two launches on the residual
(:class:`kgs.ops.postnorm.PostNorm`). Latent attention is :class:`kgs.serve.hybrid.LatentMixer`,
differential attention runs on the head pages of :mod:`kgs.ops.paged`. Weights are kept once
per layer that has its own; every layer has its own cache pages and convolution state.

``dtype="float32"``: the same steps with fp32 weights, activations and cache and the plain
attention kernels.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from kgs.models.ruruzen import LatentSpec
from kgs.models.vumalix import DiffAttentionSpec, VumalixConfig
from kgs.ops import decode as D
from kgs.ops.activation import poly_norm, softcap
from kgs.ops.latent import LatentCache
from kgs.ops.paged import Differential, paged_heads, paged_rows, paged_tiles
from kgs.ops.postnorm import MAX_WIDTH, Conv, ConvState, PostNorm, Sublayer
from kgs.ops.talking import HeadNorm, HeadPages, Heads, Temperature, write_kv

from .hybrid import LatentMixer, latent_row
from .nokipel import ChunkedGeometry, input_matrix, output_matrix
from .ragged import DTYPES, Batch, RaggedModel, Weights, _pad, pad64, pad256, padk
from .trace import TRACE as T


def attention_heads(m: DiffAttentionSpec, dtype) -> Heads:
    return paged_heads(m.heads, m.kv_heads, m.dim, m.vdim, dtype, maps=2)


# -------------------------------------------------------------------- sublayers
class DifferentialMixer:
    def __init__(self, model, i: int, m: DiffAttentionSpec, w: Weights):
        p, wp = f"l{i}.mix.", model.wp
        self.layer, self.m, self.heads = i, m, attention_heads(m, w.dtype)
        h = self.heads
        self.geo = ChunkedGeometry(h, 0)
        seg = h.dkp // 2
        win, self.offs = input_matrix(w, p, (("q", 2 * m.heads, m.dim, seg), ("k", 2 * m.kv_heads, m.dim, seg),
                                             ("v", m.kv_heads, m.vdim, h.dvp)), wp)
        self.win = w.proj(win)
        self.norm = HeadNorm(*(_pad(w.f32(f"{p}{n}.norm"), seg).contiguous() for n in "qk"), m.dim, model.cfg.eps)
        self.temperature = Temperature(m.temp_coef, m.temp_every)
        a, b = (float(torch.exp((w.w[f"{p}lq{j}"].double() * w.w[f"{p}lk{j}"].double()).sum())) for j in (1, 2))
        self.diff = Differential(a - b + m.diff, 1.0 - m.diff, m.vdim, model.cfg.eps)
        self.o = w.proj(output_matrix(w, p + "o", m.heads, m.vdim, h.dvp, wp, m.heads * h.dvp))

    def __call__(self, model, h: torch.Tensor, b: Batch, pages: torch.Tensor) -> torch.Tensor:
        hd, m, plan = self.heads, self.m, b.plans[self.geo]
        z = self.win(h)
        write_kv(z, None, pages, b.slots, hd, self.offs[1], self.offs[2], pos=b.pos, norm=self.norm,
                 temperature=self.temperature)
        T.op(f"L{self.layer} attention projections")
        a = torch.empty((h.shape[0], hd.heads * hd.dvp), dtype=h.dtype, device=h.device)
        if plan.tiles is not None:
            paged_tiles(z, pages, hd, m.scale, 0, plan.tiles, a, self.diff)
        if plan.rows is not None:
            paged_rows(z, pages, hd, m.scale, 0, plan.rows, a, self.diff)
        T.op(f"L{self.layer} attention")
        return self.o(a)


class PolyFF:
    def __init__(self, model, i: int, ff: int, w: Weights):
        p, fp = f"l{i}.mlp.", padk(ff)
        self.layer, self.ff, self.eps = i, ff, model.cfg.eps
        self.up, self.down = w.proj(w.mat(p + "up", fp, model.wp)), w.proj(w.mat(p + "down", model.wp, fp))
        self.act = w.f32(p + "act")

    def __call__(self, h: torch.Tensor) -> torch.Tensor:
        y = self.down(poly_norm(self.up(h), self.act, self.ff, self.eps))
        T.op(f"L{self.layer} feed-forward")
        return y


@dataclass
class Layer:
    """What a layer computes with; layers that share weights share it."""
    mixer: LatentMixer | DifferentialMixer
    ff: PolyFF | None
    conv: Conv
    gains: tuple[float, float]   # of the norms behind the mixer and the feed-forward


# ------------------------------------------------------------------------ model
class VumalixModel(RaggedModel):
    def __init__(self, cfg: VumalixConfig, device="cuda", dtype: str = "bfloat16", seed: int = 0,
                 num_pages: int = 1024, state_slots: int = 256, max_len: int = 8192, weights: dict | None = None,
                 packed_decode: bool = True):
        super().__init__()
        self.cfg, self.device, self.dtype = cfg, torch.device(device), DTYPES[dtype]
        self.has_state, self.max_len = cfg.has_state, max_len
        self.wp = pad256(cfg.width)
        if self.wp > MAX_WIDTH:
            raise ValueError(f"width {cfg.width} is above {MAX_WIDTH}")
        raw = weights if weights is not None else cfg.load_weights(seed, self.device)
        w = Weights(raw, self.device, self.dtype, packed_decode)
        if self.dtype == torch.bfloat16:
            D.reserve_workspace(self.device)  # split-K partials, before any hipGraph capture
        self.embed = w.mat("embed", cfg.vocab, self.wp)
        self.head = w.proj(w.mat("head", pad64(cfg.vocab), self.wp))
        self.final_gain = float(raw["final.norm"])
        own = {i: self._layer(i, w) for i in cfg.owners}
        self.layers = [own[x.owner] for x in cfg.layers]
        self.geometries = {x.mixer.geo for x in own.values()}
        rows, heads = self._latents(cfg), self._heads(cfg, self.dtype)
        self.pages = LatentCache(rows, num_pages, self.dtype, self.device).pages
        self.pages |= HeadPages(heads, num_pages, self.dtype, self.device).pages
        # slot 0 is the null slot of padded decode rows
        self.state = [ConvState(cfg.taps, self.wp, state_slots + 1, self.device) if cfg.has_state else None
                      for _ in cfg.layers]

    def _layer(self, i: int, w: Weights) -> Layer:
        x = self.cfg.layers[i]
        make = LatentMixer if isinstance(x.mixer, LatentSpec) else DifferentialMixer
        gain = lambda n: float(w.w[f"l{i}.norm{n}"])  # noqa: E731
        return Layer(make(self, i, x.mixer, w), None if x.ff is None else PolyFF(self, i, x.ff, w),
                     Conv(w.f32(f"l{i}.canon1"), self.wp), (gain(1), 0.0 if x.ff is None else gain(2)))

    @staticmethod
    def _latents(cfg: VumalixConfig) -> dict[int, int]:
        return {i: latent_row(x.mixer) for i, x in enumerate(cfg.layers) if isinstance(x.mixer, LatentSpec)}

    @staticmethod
    def _heads(cfg: VumalixConfig, dtype) -> dict[int, Heads]:
        return {i: attention_heads(x.mixer, dtype) for i, x in enumerate(cfg.layers)
                if isinstance(x.mixer, DiffAttentionSpec)}

    @classmethod
    def for_engine(cls, cfg: VumalixConfig, ec, device, backend: str, num_pages: int) -> "VumalixModel":
        cls.check_engine(ec, backend)
        if ec.prefix_caching and cfg.has_state:
            raise ValueError("prefix caching shares cache pages, not recurrent state: off for this model")
        return cls(cfg, device=device, dtype=ec.dtype, seed=ec.seed, num_pages=num_pages, state_slots=ec.max_batch,
                   max_len=ec.max_model_len, packed_decode=ec.packed_decode)

    @classmethod
    def memory(cls, cfg: VumalixConfig, dtype: str, slots: int) -> dict:
        """Bytes of the weights, of all state slots and of one page (engine sizing)."""
        dt = DTYPES[dtype]
        state = len(cfg.layers) * ConvState.bytes_per_slot(cfg.taps, pad256(cfg.width)) if cfg.has_state else 0
        page = LatentCache.bytes_per_page(cls._latents(cfg), dt.itemsize) + HeadPages.bytes_per_page(cls._heads(cfg, dt), dt.itemsize)
        return {"weights": 3 * cls._weight_bytes(cfg, dt), "state": (slots + 1) * state, "page": page}

    @staticmethod
    def _weight_bytes(cfg: VumalixConfig, dtype) -> int:
        from kgs.models.vumalix import tensor_shapes

        return dtype.itemsize * sum(int(np.prod(s)) for s in tensor_shapes(cfg).values())

    def weight_bytes(self) -> int:
        return self._weight_bytes(self.cfg, self.dtype)

    # ------------------------------------------------------------------ forward
    @torch.no_grad()
    def forward(self, b: Batch) -> torch.Tensor:
        """Runs the batch; fp32 logits ``[rows wanted, vocab]``."""
        cfg = self.cfg
        res = PostNorm(b.tokens, b.seqs, cfg.width, self.wp, cfg.eps, self.dtype)
        h = res.start(self.embed, self.layers[0].conv, self.state[0])
        for i, layer in enumerate(self.layers):
            # the inputs that the mixer has read are kept by the next launch on the residual
            y, save = Sublayer(layer.mixer(self, h, b, self.pages[i]), layer.gains[0]), self.state[i]
            if layer.ff is not None:
                h = res.add(y, save=save)
                T.op(f"L{i} residual")
                y, save = Sublayer(layer.ff(h), layer.gains[1]), None
            if i + 1 < len(self.layers):
                h = res.add(y, self.layers[i + 1].conv, self.state[i + 1], save)
            else:
                h = res.close(y, self.final_gain, save)
            T.op(f"L{i} residual")
            if self.on_layer is not None:
                self.on_layer(i, res.x[:, :cfg.width])
        if b.logit_rows is not None:
            if b.logit_rows.shape[0] == 0:
                return torch.empty((0, cfg.vocab), dtype=torch.float32, device=self.device)
            h = h.index_select(0, b.logit_rows)
        logits = softcap(self.head(h), cfg.vocab, 0.0)
        T.op("logits")
        return logits
