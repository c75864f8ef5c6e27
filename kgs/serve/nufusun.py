"""Serving model of parallel layers of talking-heads attention and mixtures of
experts (:mod:`kgs.models.nufusun`).

Every step is one ragged batch (:class:`kgs.serve.ragged.Batch`): the projections'
biases are added where keys and values go to their pages, prompt portions attend in
tiles of 16 or 32 queries, decoded tokens and short portions row by row with the context
split over the CUs. A layer's two sublayers read the same normed input; one launch
(:func:`kgs.ops.residual.residual_add`) adds both to the fp32 residual, gathering
every token's expert rows, and produces the next layer's input.

``dtype="float32"``: the same steps with fp32 weights, activations and cache, the
plain attention kernel and fp32 grouped products.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from kgs.models.nufusun import AttentionSpec, ExpertsSpec, NufusunConfig
from kgs.ops import decode as D
from kgs.ops import moe as M
from kgs.ops.activation import Gate, softcap
from kgs.ops.decode import PAGE
from kgs.ops.residual import MAX_WIDTH, ExpertRows, Norm, residual_add, residual_embed
from kgs.ops.talking import (HeadPages, Heads, QueryRows, QueryTiles, TalkingWeights, attention_rows,
                             attention_tiles, heads_of, split_count, tile_items, write_kv)

from .ragged import DTYPES, Batch, HostPack, RaggedModel, Weights, _pad, pad64, pad128, pad256
from .trace import TRACE as T

TILE_MIN = 16  # shorter portions run row by row


def attention_heads(m: AttentionSpec, dtype) -> Heads:
    return heads_of(m.heads, m.kv_heads, m.dim, m.vdim, dtype)


# ------------------------------------------------------------------------ plans
@dataclass
class TalkingPlan:
    rows: QueryRows | None
    tiles: QueryTiles | None


@dataclass(frozen=True)
class Geometry:
    """What an attention launch plan depends on."""
    heads: Heads

    def host_plan(self, pk: HostPack, row0, n, pos0, bt, row_seq, pos, refs):
        """Splits the sequences between tiles and rows and lays out both launches;
        returns the plan's builder, to be called once ``pk`` is sent."""
        tiled = (n >= TILE_MIN) & self.heads.tiled
        rows = tiles = None
        if not tiled.all():
            at = np.flatnonzero(~tiled[row_seq])
            whole = len(at) == len(row_seq)
            pages = int(pos[at].max()) // PAGE + 1
            rows = ({"tok_seq": refs[2] if whole else pk.add(row_seq[at]),
                     "tok_pos": refs[9] if whole else pk.add(pos[at]),
                     "rows": None if whole else pk.add(at)}, len(at), split_count(len(at), pages))
        if tiled.any():
            sel = np.flatnonzero(tiled)
            items, merges = tile_items([(row0[s], s, pos0[s], n[s]) for s in sel], self.heads.tile)
            tiles = (pk.add(items), pk.add(merges) if len(merges) else None, int(merges[:, 3].sum()))

        def build(get):
            r = None
            if rows is not None:
                r = QueryRows(n=rows[1], bt=get(refs[7]), nsplit=rows[2],
                              **{k: None if v is None else get(v) for k, v in rows[0].items()})
            if tiles is None:
                return TalkingPlan(r, None)
            items, merges, parts = tiles
            return TalkingPlan(r, QueryTiles(get(items), get(refs[7]), None if merges is None else get(merges), parts))

        return build

    def decode_plan(self, f, nb, positions, block_tables):
        return TalkingPlan(QueryRows(nb, block_tables, f["ar"], positions, None,
                                     split_count(nb, block_tables.shape[1])), None)


# -------------------------------------------------------------------- sublayers
class TalkingMixer:
    def __init__(self, model, i: int, m: AttentionSpec, w: Weights):
        p = f"l{i}.mix."
        cfg, wp = model.cfg, model.wp
        self.layer, self.heads = i, attention_heads(m, w.dtype)
        h = self.heads
        self.geo = Geometry(h)

        def rows(t, n, d, dp):  # [n d, ..] -> [n dp, ..], every head padded
            return _pad(t.reshape(n, d, -1), dp, t.shape[-1]).reshape(n * dp, -1)

        mats, biases, self.offs, at = [], [], [], 0
        for name, n, d, dp in (("q", m.heads, m.dim, h.dkp), ("k", m.kv_heads, m.dim, h.dkp),
                               ("v", m.kv_heads, m.vdim, h.dvp)):
            t = rows(w.w[p + name].to(w.device).to(w.dtype), n, d, dp)
            mats.append(_pad(t, pad64(n * dp), wp))
            biases.append(rows(w.f32(f"{p}{name}.b")[:, None], n, d, dp).reshape(-1))
            self.offs.append(at)
            at += mats[-1].shape[0]
        if at > 1024 and at % 256:  # whole 256-wide GEMM tiles
            mats.append(torch.zeros((256 - at % 256, wp), dtype=w.dtype, device=w.device))
        self.win = w.proj(torch.cat(mats).contiguous())
        self.bias = torch.cat(biases).contiguous()
        self.talk = TalkingWeights(h, w.w[p + "talk"], w.w[p + "temp"], w.w[p + "rel"], m.scale, m.bias_max, w.device)
        o = w.w[p + "o"].to(w.device).to(w.dtype).reshape(cfg.width, m.heads, m.vdim)
        self.o = w.proj(_pad(_pad(o, h.dvp).reshape(cfg.width, m.heads * h.dvp), wp, m.heads * h.dvp))
        self.o_bias = _pad(w.f32(p + "o.b"), wp)

    def __call__(self, model, h: torch.Tensor, b: Batch) -> torch.Tensor:
        hd, plan = self.heads, b.plans[self.geo]
        z = self.win(h)
        pages = model.cache.pages[self.layer]
        write_kv(z, self.bias, pages, b.slots, hd, self.offs[1], self.offs[2])
        T.op(f"L{self.layer} attention projections")
        a = torch.empty((h.shape[0], hd.heads * hd.dvp), dtype=h.dtype, device=h.device)
        if plan.tiles is not None:
            attention_tiles(z, pages, self.talk, plan.tiles, a)
        if plan.rows is not None:
            attention_rows(z, pages, self.talk, plan.rows, a)
        T.op(f"L{self.layer} attention")
        return self.o(a)


class ExpertsFF:
    def __init__(self, model, i: int, m: ExpertsSpec, w: Weights, counts: torch.Tensor):
        p, wp, fp = f"l{i}.mlp.", model.wp, pad128(m.ff)
        self.layer, self.m, self.counts = i, m, counts
        self.router = w.mat(p + "router", M.router_rows(m.experts), wp).contiguous()
        self.gate_up = torch.stack([torch.cat([w.mat(f"{p}e{e}.{n}", fp, wp) for n in ("gate", "up")])
                                    for e in range(m.experts)])
        self.down = torch.stack([w.mat(f"{p}e{e}.down", wp, fp) for e in range(m.experts)])

    def __call__(self, model, h: torch.Tensor, b: Batch) -> ExpertRows:
        m = self.m
        c = M.route(h, self.router, self.counts, m.top, b.slots)
        p = M.plan(c, M.tile_rows(h.shape[0], m.top, m.experts, h.dtype))
        T.op(f"L{self.layer} router")
        y = M.down(M.gate_up(h, self.gate_up, p, Gate("clamped", m.limit)), self.down, p)
        T.op(f"L{self.layer} experts")
        return ExpertRows(y, p.pos)


# ------------------------------------------------------------------------ model
class NufusunModel(RaggedModel):
    def __init__(self, cfg: NufusunConfig, device="cuda", dtype: str = "bfloat16", seed: int = 0,
                 num_pages: int = 1024, weights: dict | None = None, packed_decode: bool = True):
        super().__init__()
        self.cfg, self.device, self.dtype = cfg, torch.device(device), DTYPES[dtype]
        self.wp = pad256(cfg.width)
        if self.wp > MAX_WIDTH:
            raise ValueError(f"width {cfg.width} is above {MAX_WIDTH}")
        raw = weights if weights is not None else cfg.load_weights(seed, self.device)
        w = Weights(raw, self.device, self.dtype, packed_decode)
        if self.dtype == torch.bfloat16:
            D.reserve_workspace(self.device)  # split-K partials, before any hipGraph capture
        self.embed = w.mat("embed", cfg.vocab, self.wp)
        self.head = w.proj(w.mat("head", pad64(cfg.vocab), self.wp))
        # tokens per expert of every layer, cleared at the start of a step
        sizes = [0 if x.mlp is None else x.mlp.experts for x in cfg.layers]
        if max(sizes) > M.MAX_EXPERTS:
            raise ValueError(f"{max(sizes)} experts are above {M.MAX_EXPERTS}")
        self.counts = torch.zeros(max(1, sum(sizes)), dtype=torch.int32, device=self.device)
        self.layers = []
        for i, (layer, c) in enumerate(zip(cfg.layers, self.counts[:sum(sizes)].split(sizes))):
            self.layers.append((TalkingMixer(self, i, layer.mixer, w),
                                None if layer.mlp is None else ExpertsFF(self, i, layer.mlp, w, c)))
        self.norms = [_pad(w.f32(f"l{i}.norm1"), self.wp).contiguous() for i in range(len(cfg.layers))]
        self.norms.append(_pad(w.f32("final.norm"), self.wp).contiguous())
        self.geometries = {mixer.geo for mixer, _ in self.layers}
        self.cache = HeadPages({i: mixer.heads for i, (mixer, _) in enumerate(self.layers)}, num_pages, self.dtype,
                               self.device)

    @classmethod
    def for_engine(cls, cfg: NufusunConfig, ec, device, backend: str, num_pages: int) -> "NufusunModel":
        cls.check_engine(ec, backend)
        return cls(cfg, device=device, dtype=ec.dtype, seed=ec.seed, num_pages=num_pages, packed_decode=ec.packed_decode)

    @staticmethod
    def memory(cfg: NufusunConfig, dtype: str, slots: int) -> dict:
        """Bytes of the weights, of all state slots and of one page (engine sizing)."""
        from kgs.models.nufusun import tensor_shapes

        dt = DTYPES[dtype]
        # the experts twice while they are stacked, the other projections with their decode copies
        n = sum(int(np.prod(s)) for s in tensor_shapes(cfg).values())
        heads = {i: attention_heads(x.mixer, dt) for i, x in enumerate(cfg.layers)}
        return {"weights": 3 * dt.itemsize * n, "state": 0, "page": HeadPages.bytes_per_page(heads, dt.itemsize)}

    def weight_bytes(self) -> int:
        from kgs.models.nufusun import tensor_shapes

        return self.dtype.itemsize * sum(int(np.prod(s)) for s in tensor_shapes(self.cfg).values())

    # ------------------------------------------------------------------ forward
    @torch.no_grad()
    def forward(self, b: Batch) -> torch.Tensor:
        """Runs the batch; fp32 logits ``[rows wanted, vocab]``."""
        cfg = self.cfg
        norm = Norm(cfg.width, cfg.eps)
        x, h = residual_embed(b.tokens, self.embed, cfg.embed_scale, self.norms[0], norm, zero=self.counts)
        for i, (mixer, ff) in enumerate(self.layers):
            a = mixer(self, h, b)
            e = None if ff is None else ff(self, h, b)
            h = residual_add(x, a, mixer.o_bias, e, self.norms[i + 1], norm, self.dtype)
            T.op(f"L{i} residual")
            if self.on_layer is not None:
                self.on_layer(i, x[:, :cfg.width])
        if b.logit_rows is not None:
            if b.logit_rows.shape[0] == 0:
                return torch.empty((0, cfg.vocab), dtype=torch.float32, device=self.device)
            h = h.index_select(0, b.logit_rows)
        logits = softcap(self.head(h), cfg.vocab, 0.0)
        T.op("logits")
        return logits
