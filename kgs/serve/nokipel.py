"""Serving model of layer stacks that mix chunked and lightning attention with dense
feed-forwards and mixtures of experts, some layers passed several times
(:mod:`kgs.models.nokipel`).

Every step is one ragged batch (:class:`kgs.serve.ragged.Batch`). A sublayer is ``h ->
mixer or feed-forward -> y`` between two launches of
:func:`kgs.ops.residual.residual_add`, which adds ``y`` (a projection, or every token's
expert rows, its identity experts' share of ``h`` and its gated shared expert) to the fp32
residual and produces the next sublayer's normed input; at the start of a later pass it
also adds the embedding output, straight from the table. Layers keep their weights
once; every *run* of a layer has cache pages or states, and expert counters, of its own.

``dtype="float32"``: the same steps with fp32 weights, activations and cache, the plain
attention kernel, the token-by-token recurrence and fp32 grouped products.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from kgs.models.nokipel import AttentionSpec, DenseSpec, ExpertsSpec, LightningSpec, NokipelConfig
from kgs.ops import decode as D
from kgs.ops import moe as M
from kgs.ops.activation import Gate, softcap
from kgs.ops.lightning import (CHUNK_DIM, Decays, LightningShape, LightningState, SegmentPlan, lightning_forward,
                               lightning_out, segment_plan)
from kgs.ops.paged import (Portions, paged_heads, paged_rows, paged_tiles, portion_items, row_splits, tile_queries,
                           visible_pages)
from kgs.ops.residual import MAX_WIDTH, Embedding, ExpertRows, Norm, Scaled, residual_add, residual_embed
from kgs.ops.talking import HeadPages, Heads, QueryRows, write_kv

from .ragged import DTYPES, Batch, HostPack, RaggedModel, Weights, _pad, pad64, pad128, pad256, padk
from .trace import TRACE as T

TILE_MIN = 16  # shorter portions run row by row


def attention_heads(m: AttentionSpec, dtype) -> Heads:
    return paged_heads(m.heads, m.kv_heads, m.dim, m.vdim, dtype)


def lightning_shape(m: LightningSpec) -> LightningShape:
    return LightningShape(m.heads, m.dim, m.vdim)


# ------------------------------------------------------------------------ plans
@dataclass
class ChunkedPlan:
    rows: QueryRows | None
    tiles: Portions | None


@dataclass(frozen=True)
class ChunkedGeometry:
    """What a launch plan of attention over head pages depends on."""
    heads: Heads
    chunk: int

    def host_plan(self, pk: HostPack, row0, n, pos0, bt, row_seq, pos, refs):
        """Splits the sequences between tiles and rows and lays out both launches;
        returns the plan's builder, to be called once ``pk`` is sent."""
        h = self.heads
        tiled = (n >= TILE_MIN) & (tile_queries(h) > 0)
        rows = items = None
        if not tiled.all():
            at = np.flatnonzero(~tiled[row_seq])
            whole = len(at) == len(row_seq)
            pages = max(visible_pages(int(p), self.chunk) for p in pos[at])
            rows = ({"tok_seq": refs[2] if whole else pk.add(row_seq[at]),
                     "tok_pos": refs[9] if whole else pk.add(pos[at]),
                     "rows": None if whole else pk.add(at)}, len(at), row_splits(len(at), h.kv_heads, h.group, pages, h.maps))
        if tiled.any():
            sel = np.flatnonzero(tiled)
            items = pk.add(portion_items([(row0[s], s, pos0[s], n[s]) for s in sel], tile_queries(h), self.chunk))

        def build(get):
            r = None
            if rows is not None:
                r = QueryRows(n=rows[1], bt=get(refs[7]), nsplit=rows[2],
                              **{k: None if v is None else get(v) for k, v in rows[0].items()})
            return ChunkedPlan(r, None if items is None else Portions(get(items), get(refs[7])))

        return build

    def decode_plan(self, f, nb, positions, block_tables):
        pages = block_tables.shape[1]
        if self.chunk:
            pages = min(pages, (self.chunk - 1) // D.PAGE + 2)
        return ChunkedPlan(QueryRows(nb, block_tables, f["ar"], positions, None,
                                     row_splits(nb, self.heads.kv_heads, self.heads.group, pages,
                                                self.heads.maps)), None)


@dataclass(frozen=True)
class LightningGeometry:
    """What a launch plan of lightning attention depends on."""
    units: int     # workgroups of one segment
    chunked: bool

    def host_plan(self, pk: HostPack, row0, n, pos0, bt, row_seq, pos, refs):
        p = segment_plan(n, self.units, self.chunked)
        whole = len(p["step"]) == len(n)
        seqs = None if whole or not len(p["step"]) else pk.add(p["step"])
        items, scans = (pk.add(p[k]) if len(p[k]) else None for k in ("items", "scans"))

        def build(get):
            opt = lambda r: None if r is None else get(r)  # noqa: E731
            return SegmentPlan(len(p["step"]), opt(seqs), opt(items), opt(scans), p["buffers"])

        return build

    def decode_plan(self, f, nb, positions, block_tables):
        return SegmentPlan(nb)


# -------------------------------------------------------------------- sublayers
def _head_rows(t: torch.Tensor, n: int, d: int, dp: int) -> torch.Tensor:
    """``[n d, ..] -> [n dp, ..]``, every head padded."""
    return _pad(t.reshape(n, d, -1), dp, t.shape[-1]).reshape(n * dp, -1)


def input_matrix(w: Weights, p: str, parts, wp: int) -> tuple[torch.Tensor, list[int]]:
    """Projections of one input (name, heads, size, padded size) as one matrix
    (:meth:`Weights.join`)."""
    return w.join([w.heads(w.w[p + name], n, d, dp) for name, n, d, dp in parts], wp)


def output_matrix(w: Weights, name: str, n: int, d: int, dp: int, wp: int, cols: int) -> torch.Tensor:
    o = w.w[name].to(w.device).to(w.dtype)
    return _pad(_pad(o.reshape(o.shape[0], n, d), dp).reshape(o.shape[0], n * dp), wp, cols)


class ChunkedMixer:
    def __init__(self, model, i: int, m: AttentionSpec, w: Weights):
        p, wp = f"l{i}.mix.", model.wp
        self.layer, self.m, self.heads = i, m, attention_heads(m, w.dtype)
        h = self.heads
        self.geo = ChunkedGeometry(h, m.chunk)
        parts = (("q", m.heads, m.dim, h.dkp), ("k", m.kv_heads, m.dim, h.dkp), ("v", m.kv_heads, m.vdim, h.dvp))
        win, self.offs = input_matrix(w, p, parts, wp)
        self.win = w.proj(win)
        self.bias = torch.cat([_head_rows(w.f32(f"{p}{n}.b")[:, None], c, d, dp).reshape(-1)
                               for n, c, d, dp in parts]).contiguous()
        self.rotary = model.rotary(m.rot_dims, m.rot_base) if m.rot_dims else None
        self.o = w.proj(output_matrix(w, p + "o", m.heads, m.vdim, h.dvp, wp, m.heads * h.dvp))

    def __call__(self, model, run: int, h: torch.Tensor, b: Batch) -> torch.Tensor:
        hd, m, plan = self.heads, self.m, b.plans[self.geo]
        z = self.win(h)
        pages = model.cache.pages[run]
        write_kv(z, self.bias, pages, b.slots, hd, self.offs[1], self.offs[2], self.rotary, b.pos)
        T.op(f"L{self.layer} attention projections")
        a = torch.empty((h.shape[0], hd.heads * hd.dvp), dtype=h.dtype, device=h.device)
        if plan.tiles is not None:
            paged_tiles(z, pages, hd, m.scale, m.chunk, plan.tiles, a)
        if plan.rows is not None:
            paged_rows(z, pages, hd, m.scale, m.chunk, plan.rows, a)
        T.op(f"L{self.layer} attention")
        return self.o(a)


class LightningMixer:
    def __init__(self, model, i: int, m: LightningSpec, w: Weights):
        p, wp = f"l{i}.mix.", model.wp
        self.layer, self.eps, self.shape = i, model.cfg.eps, lightning_shape(m)
        s = self.shape
        self.geo = LightningGeometry(m.heads * s.slabs, w.dtype == torch.bfloat16 and m.dim <= CHUNK_DIM)
        parts = [(n, m.heads, m.dim, s.kp) for n in "qk"] + [(n, m.heads, m.vdim, s.vp) for n in "vg"]
        win, offs = input_matrix(w, p, parts, wp)
        self.win = w.proj(win)
        self.offs, self.og = tuple(offs[:3]), offs[3]
        self.decays = Decays(m.decay, w.device)
        self.count, n = m.heads * m.vdim, m.heads * s.vp
        self.norm = _head_rows(w.f32(p + "norm")[:, None], m.heads, m.vdim, s.vp).reshape(-1).contiguous()
        self.ld = padk(n)
        self.o = w.proj(output_matrix(w, p + "o", m.heads, m.vdim, s.vp, wp, self.ld))

    def __call__(self, model, run: int, h: torch.Tensor, b: Batch) -> torch.Tensor:
        z = self.win(h)
        T.op(f"L{self.layer} lightning projections")
        o = lightning_forward(z, self.offs, self.shape, self.decays, model.state[run], b.seqs, b.plans[self.geo])
        y = lightning_out(o, self.norm, z[:, self.og:self.og + o.shape[1]], self.count, self.eps, self.ld)
        T.op(f"L{self.layer} lightning attention")
        return self.o(y)


class DenseFF:
    def __init__(self, model, i: int, m: DenseSpec, w: Weights):
        p, fp = f"l{i}.mlp.", padk(m.ff)
        self.layer = i
        self.gate_up = w.proj(torch.cat([w.mat(p + n, fp, model.wp) for n in ("gate", "up")]), gated=Gate("clamped", m.limit))
        self.down = w.proj(w.mat(p + "down", model.wp, fp))

    def __call__(self, model, run: int, h: torch.Tensor, b: Batch) -> dict:
        y = self.down(self.gate_up(h))
        T.op(f"L{self.layer} feed-forward")
        return {"a": y}


class ExpertsFF:
    def __init__(self, model, i: int, m: ExpertsSpec, w: Weights):
        p, wp, fp = f"l{i}.mlp.", model.wp, pad128(m.ff)
        self.layer, self.m = i, m
        self.route = M.Softmax(m.experts, m.identity, m.top, m.groups, m.keep, m.scale)
        n = m.experts + m.identity
        router = [w.mat(p + "router", n, wp)] + ([w.mat(p + "shared.sg", 1, wp)] if m.shared_ff else [])
        router = torch.cat(router)
        self.router = _pad(router, M.router_rows(router.shape[0]), wp).contiguous()
        self.correction = w.f32(p + "correction")
        self.gate_up = torch.stack([torch.cat([w.mat(f"{p}e{e}.{n}", fp, wp) for n in ("gate", "up")])
                                    for e in range(m.experts)])
        self.down = torch.stack([w.mat(f"{p}e{e}.down", wp, fp) for e in range(m.experts)])
        self.shared = None
        if m.shared_ff:
            sp = padk(m.shared_ff)
            self.shared = (w.proj(torch.cat([w.mat(f"{p}shared.{n}", sp, wp) for n in ("gate", "up")]), gated="silu"),
                           w.proj(w.mat(p + "shared.down", wp, sp)))

    def __call__(self, model, run: int, h: torch.Tensor, b: Batch) -> dict:
        m = self.m
        c, ident, gate = M.route_softmax(h, self.router, model.counts[run], self.route, self.correction, b.slots,
                                         gate=self.shared is not None)
        p = M.plan(c, M.tile_rows(h.shape[0], m.top, m.experts, h.dtype))
        T.op(f"L{self.layer} router")
        y = M.down(M.gate_up(h, self.gate_up, p, Gate("silu")), self.down, p)
        T.op(f"L{self.layer} experts")
        scaled = [] if ident is None else [Scaled(h, ident)]
        if self.shared is not None:
            scaled.append(Scaled(self.shared[1](self.shared[0](h)), gate))
            T.op(f"L{self.layer} shared expert")
        return {"experts": ExpertRows(y, p.pos), "scaled": scaled}


# ------------------------------------------------------------------------ model
class NokipelModel(RaggedModel):
    def __init__(self, cfg: NokipelConfig, device="cuda", dtype: str = "bfloat16", seed: int = 0,
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
        self.norm = Norm(cfg.width, cfg.eps, cfg.norm_groups, 0.0)
        self.embed = w.mat("embed", cfg.vocab, self.wp)
        self.head = w.proj(w.mat("head", pad64(cfg.vocab), self.wp))
        self.mixers, self.ffs = [], []
        for i, layer in enumerate(cfg.layers):
            self.mixers.append((ChunkedMixer if isinstance(layer.mixer, AttentionSpec) else LightningMixer)(self, i, layer.mixer, w))
            f = layer.mlp
            self.ffs.append(None if f is None else (DenseFF if isinstance(f, DenseSpec) else ExpertsFF)(self, i, f, w))
        norm = lambda name: _pad(w.f32(name), self.wp).contiguous()  # noqa: E731
        self.norms = [(norm(f"l{i}.norm1"), None if layer.mlp is None else norm(f"l{i}.norm2"))
                      for i, layer in enumerate(cfg.layers)]
        self.final_norm = norm("final.norm")
        self.geometries = {m.geo for m in self.mixers}
        self.runs = cfg.runs
        # tokens per expert of every run, cleared at the start of a step
        sizes = [x.mlp.experts if isinstance(x.mlp, ExpertsSpec) else 0 for x in (cfg.layers[i] for i, _ in self.runs)]
        if any(isinstance(x.mlp, ExpertsSpec) and x.mlp.experts + x.mlp.identity > M.MAX_EXPERTS for x in cfg.layers):
            raise ValueError(f"more than {M.MAX_EXPERTS} experts")
        self.all_counts = torch.zeros(max(1, sum(sizes)), dtype=torch.int32, device=self.device)
        self.counts = self.all_counts[:sum(sizes)].split(sizes)
        self.cache = HeadPages(self._heads(cfg, self.dtype), num_pages, self.dtype, self.device)
        # slot 0 is the null slot of padded decode rows
        self.state = {r: LightningState(s, state_slots + 1, self.device) for r, s in self._shapes(cfg).items()}

    @staticmethod
    def _heads(cfg: NokipelConfig, dtype) -> dict[int, Heads]:
        return {r: attention_heads(cfg.layers[i].mixer, dtype) for r, (i, _) in enumerate(cfg.runs)
                if isinstance(cfg.layers[i].mixer, AttentionSpec)}

    @staticmethod
    def _shapes(cfg: NokipelConfig) -> dict[int, LightningShape]:
        return {r: lightning_shape(cfg.layers[i].mixer) for r, (i, _) in enumerate(cfg.runs)
                if isinstance(cfg.layers[i].mixer, LightningSpec)}

    @classmethod
    def for_engine(cls, cfg: NokipelConfig, ec, device, backend: str, num_pages: int) -> "NokipelModel":
        cls.check_engine(ec, backend)
        if ec.prefix_caching and cfg.has_state:
            raise ValueError("prefix caching shares cache pages, not recurrent state: off for this model")
        return cls(cfg, device=device, dtype=ec.dtype, seed=ec.seed, num_pages=num_pages, state_slots=ec.max_batch,
                   max_len=ec.max_model_len, packed_decode=ec.packed_decode)

    @classmethod
    def memory(cls, cfg: NokipelConfig, dtype: str, slots: int) -> dict:
        """Bytes of the weights, of all state slots and of one page (engine sizing)."""
        dt = DTYPES[dtype]
        state = sum(LightningState.bytes_per_slot(s) for s in cls._shapes(cfg).values())
        # the experts twice while they are stacked, the other projections with their decode copies
        return {"weights": 3 * cls._weight_bytes(cfg, dt), "state": (slots + 1) * state,
                "page": HeadPages.bytes_per_page(cls._heads(cfg, dt), dt.itemsize) or 1}

    @staticmethod
    def _weight_bytes(cfg: NokipelConfig, dtype) -> int:
        from kgs.models.nokipel import tensor_shapes

        return dtype.itemsize * sum(int(np.prod(s)) for s in tensor_shapes(cfg).values())

    def weight_bytes(self) -> int:
        return self._weight_bytes(self.cfg, self.dtype)

    # ------------------------------------------------------------------ forward
    @torch.no_grad()
    def forward(self, b: Batch) -> torch.Tensor:
        """Runs the batch; fp32 logits ``[rows wanted, vocab]``."""
        cfg = self.cfg
        again = Embedding(b.tokens, self.embed, cfg.embed_scale)

        def add(w, a=None, experts=None, scaled=(), embedding=None):
            return residual_add(x, a, None, experts, w, self.norm, self.dtype, scaled=scaled, embedding=embedding)

        x, h = residual_embed(b.tokens, self.embed, cfg.embed_scale, self.norms[self.runs[0][0]][0], self.norm,
                              zero=self.all_counts)
        for r, (i, _) in enumerate(self.runs):
            nxt, restart = self.runs[r + 1] if r + 1 < len(self.runs) else (None, False)
            after = self.final_norm if nxt is None else self.norms[nxt][0]
            y = {"a": self.mixers[i](self, r, h, b)}
            if self.ffs[i] is not None:
                h = add(self.norms[i][1], **y)
                T.op(f"L{i} residual")
                y = self.ffs[i](self, r, h, b)
            if self.on_layer is not None:
                h = add(after, **y)
                self.on_layer(r, x[:, :cfg.width])
                y = {}
            if self.on_layer is None or restart:
                h = add(after, **y, embedding=again if restart else None)
            T.op(f"L{i} residual")
        if b.logit_rows is not None:
            if b.logit_rows.shape[0] == 0:
                return torch.empty((0, cfg.vocab), dtype=torch.float32, device=self.device)
            h = h.index_select(0, b.logit_rows)
        logits = softcap(self.head(h), cfg.vocab, 0.0)
        T.op("logits")
        return logits
