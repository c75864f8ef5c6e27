"""Serving model of layer stacks that mix latent attention and delta-rule mixers
over hyper-connected residual streams (:mod:`kgs.models.ruruzen`).

Every step -- prompts, prompt portions, mixed steps, decode -- is one ragged batch
(:class:`kgs.serve.ragged.Batch`). The same :meth:`HybridModel.forward` runs all of
them; decode steps (one token per sequence) have fixed shapes and are captured in
hipGraphs by the engine.

A sublayer is ``h -> mixer or feed-forward -> y`` between two launches of
:func:`kgs.ops.hyper.hyper_step`, which writes ``y`` back into the fp32 streams and
produces the next sublayer's normed input in one pass. Weights are laid out once
at load: the projections of one input fused into one matrix, every dimension
that a GEMM sees padded with zeros to a multiple of 64 (larger ones of 128).

``dtype="float32"``: the same steps with fp32 weights, activations and caches.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from kgs.models.ruruzen import DeltaSpec, LatentSpec, RuruzenConfig
from kgs.ops.activation import softcap
from kgs.ops import decode as D
from kgs.ops.decode import PAGE
from kgs.ops.delta import DeltaShape, DeltaState, delta_forward, delta_out
from kgs.ops.hyper import MAX_STREAMS, hyper_embed, hyper_step
from kgs.ops.latent import (LatentCache, LatentRows, head_proj, latent_attention, latent_norm, mfma_sizes,
                            padded_latent, padded_rot, split_count, waves_for, window_pages)
from kgs.ops.linear import Projection
from kgs.ops.transformer import attention_ragged

from .ragged import DTYPES, Batch, HostPack, RaggedModel, Weights, _pad, pad64, padk
from .trace import TRACE as T

EXPAND_MIN = 16  # shorter portions are not worth the expansion's launches
QBLOCK = 128  # query rows of one attention_ragged item


def latent_row(m: LatentSpec) -> int:
    """Columns of a cache row."""
    return padded_latent(m.kv_rank) + padded_rot(m.rot_dim)


def latent_sizes(cfg: RuruzenConfig) -> dict[int, int]:
    """Columns of a cache row of every layer that caches a latent."""
    return {i: latent_row(x.mixer) for i, x in enumerate(cfg.layers)
            if isinstance(x.mixer, LatentSpec) and x.mixer.kv_from is None}


def delta_shape(m: DeltaSpec) -> DeltaShape:
    return DeltaShape(m.heads, m.kv_heads, m.dim, m.vdim, m.conv)


# ------------------------------------------------------------------------ plans
@dataclass
class Expanded:
    """Portions that attend over expanded keys and values."""
    items: torch.Tensor        # attention_ragged items
    ctx_slots: torch.Tensor    # cache slot of every key, the sequences one after another (int64)


@dataclass
class LatentPlan:
    absorbed: LatentRows | None
    expanded: Expanded | None


@dataclass(frozen=True)
class Geometry:
    """What a latent-attention launch plan depends on."""
    heads: int
    rp: int
    hd: int                    # head size of the expanded form, 0: absorbed only
    window: int = 0            # 0: every earlier key

    def pages(self, pages: int, queries: int) -> int:
        """Most of ``pages`` that a tile of ``queries`` tokens reads."""
        return min(pages, window_pages(self.window, queries)) if self.window else pages

    def expand(self, n: int, pos0: int) -> bool:
        """Whether a portion of ``n`` tokens after ``pos0`` runs on expanded keys and
        values. Per head that expands every context token (``4 rp hd`` flops each)
        where the absorbed form maps every query token (as many), and pays ``4 hd``
        per (query, key) pair where the absorbed form pays ``4 rp``."""
        if self.window:
            ctx = min(pos0, self.window - 1)
            grow = min(n, max(0, self.window - pos0))  # tokens that see one key more than the last
            pairs = grow * (pos0 + 0.5 * grow) + (n - grow) * self.window
        else:
            ctx, pairs = pos0, n * (pos0 + 0.5 * n)
        return self.hd > 0 and n >= EXPAND_MIN and ctx * self.rp * self.hd < (self.rp - self.hd) * pairs

    def lay_out(self, pk: HostPack, row0, n, pos0, bt, row_seq, pos, refs):
        """Splits the sequences between the absorbed and the expanded form and adds
        both launches' arrays to ``pk``."""
        big = np.array([self.expand(int(x), int(p)) for x, p in zip(n, pos0)], bool)
        absorbed = expanded = None
        sel = np.flatnonzero(~big)
        if len(sel):
            ns = n[sel]
            q0 = np.cumsum(ns) - ns
            rows = ns * self.heads
            waves = waves_for(int(rows.max()), self.rp)
            tiles = -(-rows // (16 * waves))
            # the tiles with the longest context first
            seq = np.repeat(np.arange(len(sel)), tiles)
            tile = np.arange(len(seq)) - np.repeat(np.cumsum(tiles) - tiles, tiles)
            end = pos0[sel][seq] + np.minimum((tile + 1) * 16 * waves, rows[seq]) // self.heads
            o = np.argsort(-end, kind="stable")
            items = np.stack([seq[o], tile[o]], 1)
            ident = len(sel) == len(n) and np.array_equal(q0, row0)
            order = None if ident else np.concatenate([np.arange(r, r + c) for r, c in zip(row0[sel], ns)])
            at = np.arange(len(row_seq)) if order is None else order
            maxp = self.pages(int((pos0[sel] + ns - 1).max()) // PAGE + 1, 16 * waves // self.heads + 2)
            absorbed = ({"q0": pk.add(q0), "n": pk.add(ns), "pos0": pk.add(pos0[sel]),
                         "bt": refs[7] if ident else pk.add(bt[sel]),
                         "tok_seq": pk.add(np.repeat(np.arange(len(sel)), ns)), "tok_pos": pk.add(pos[at]),
                         "rows": None if order is None else pk.add(order), "items": pk.add(items)},
                        {"nt": int(ns.sum()), "ntiles": len(items), "tiles": 0, "waves": waves,
                         "nsplit": split_count(len(items), maxp, self.rp)})
        sel = np.flatnonzero(big)
        if len(sel):
            items, ctx, base = [], [], 0
            for s in sel:
                first = max(0, int(pos0[s]) - self.window + 1) if self.window else 0
                p = np.arange(first, int(pos0[s] + n[s]))
                ctx.append(bt[s][p // PAGE].astype(np.int64) * PAGE + p % PAGE)
                for q in range(0, int(n[s]), QBLOCK):
                    items.append((row0[s] + q, base, pos0[s] - first + q, min(QBLOCK, n[s] - q)))
                base += len(p)
            items = np.array(items, np.int64)
            items = items[np.argsort(-(items[:, 2] + items[:, 3]), kind="stable")]
            expanded = (pk.add(items), pk.add(np.concatenate(ctx)))
        return absorbed, expanded

    def host_plan(self, pk: HostPack, *layout):
        """The builder of the plan, to be called once ``pk`` is sent."""
        absorbed, expanded = self.lay_out(pk, *layout)

        def build(get):
            a = e = None
            if absorbed is not None:
                r, shape = absorbed
                a = LatentRows(**{k: (None if v is None else get(v)) for k, v in r.items()}, **shape)
            if expanded is not None:
                e = Expanded(get(expanded[0]), get(expanded[1]).long())
            return LatentPlan(a, e)

        return build

    def decode_plan(self, f, nb, positions, block_tables):
        waves = waves_for(self.heads, self.rp)
        tiles = -(-self.heads // (16 * waves))
        return LatentPlan(LatentRows(
            nt=nb, q0=f["ar"], n=f["one"], pos0=positions, bt=block_tables, tok_seq=f["ar"], tok_pos=positions,
            rows=None, items=None, ntiles=nb * tiles, tiles=tiles, waves=waves,
            nsplit=split_count(nb * tiles, self.pages(block_tables.shape[1], 1), self.rp)), None)


# -------------------------------------------------------------------- sublayers
def neighbours(t: torch.Tensor, dim: int) -> torch.Tensor:
    """Rows whose first half turns with the second one's, reordered to neighbouring pairs (a
    score does not depend on the order that q and k share)."""
    a, b = t.chunk(2, dim)
    return torch.stack([a, b], dim + 1).flatten(dim, dim + 1)


class LatentMixer:
    """``pages`` of a call: the cache of the layer (default: the model's, by layer)."""

    def __init__(self, model, i: int, m: LatentSpec, w: Weights):
        p = f"l{i}.mix."
        cfg = model.cfg
        self.m, self.owner = m, i if m.kv_from is None else m.kv_from
        self.layer = i
        self.eps = cfg.eps
        H, own = m.heads, m.kv_from is None
        rp, hr = padded_latent(m.kv_rank), padded_rot(m.rot_dim)
        both = max(m.dim, m.vdim)
        hd = (64 if both <= 64 else 128 if both <= 128 else 0) if w.dtype == torch.bfloat16 and mfma_sizes(32, hr) else 0
        self.hq, self.hv, self.hr = (hd, hd, hr) if hd else (pad64(m.dim), pad64(m.vdim), hr)
        self.gate_cols = H * self.hv if m.gate_each else H
        dkv = w.w[p + "dkv"] if own else None
        parts = [w.w[p + "dq"], w.heads(w.w[p + "g"], H, m.vdim, self.hv) if m.gate_each else w.w[p + "g"]]
        parts += [dkv[:m.kv_rank]] if own else []
        parts += [neighbours(dkv[m.kv_rank:], 0)] if own and hr else []
        win, offs = w.join(parts, model.wp)
        self.win = w.proj(win)
        self.oq, self.og = offs[0], offs[1]
        self.oc = offs[2] if own else 0
        self.okr = offs[3] if own and hr else 0
        self.rotary = model.rotary(m.rot_dim, m.rot_base) if hr else None
        self.wq = w.f32(p + "dq.norm")
        self.wc = w.f32(p + "dkv.norm") if own else None
        self.qp = padk(m.q_rank)
        self.geo = Geometry(m.heads, rp, hd, m.window)

        def heads(name, d, dp, rank, rankp):
            t = w.w[p + name].to(w.device).to(w.dtype).reshape(H, d, rank)
            return _pad(t, dp, rankp)

        uq = w.w[p + "uq"].to(w.device).to(w.dtype).reshape(H, m.dim + m.rot_dim, m.q_rank)
        uq = torch.cat([_pad(uq[:, :m.dim], self.hq, self.qp)]
                       + ([_pad(neighbours(uq[:, m.dim:], 1), hr, self.qp)] if hr else []), 1)
        self.uq = w.proj(uq.reshape(-1, self.qp))
        uk = heads("uk", m.dim, self.hq, m.kv_rank, rp)
        self.uv = heads("uv", m.vdim, self.hv, m.kv_rank, rp).contiguous()          # [H, HV, RP]
        self.ukt = uk.transpose(1, 2).contiguous()                                  # [H, RP, HQ]
        self.ukv = Projection(torch.cat([uk.reshape(-1, rp), self.uv.reshape(-1, rp)]), pack=False) if hd else None
        o = w.w[p + "o"].to(w.device).to(w.dtype).reshape(cfg.width, H, m.vdim)
        self.o = w.proj(_pad(_pad(o, self.hv).reshape(cfg.width, H * self.hv), model.wp, H * self.hv))

    def __call__(self, model, h: torch.Tensor, b: Batch, pages: torch.Tensor | None = None) -> torch.Tensor:
        m, geo, hr = self.m, self.geo, self.hr
        z = self.win(h)
        if pages is None:
            pages = model.cache.pages[self.owner]
        cq = latent_norm(z, self.oq, self.wq, self.qp, self.oc, self.wc, pages if self.wc is not None else None,
                         b.slots, self.eps, geo.rp, self.okr, self.rotary, b.pos)
        q = self.uq(cq)
        T.op(f"L{self.layer} latent projections")
        gate = z[:, self.og:self.og + self.gate_cols]
        plan = b.plans[geo]
        a = torch.empty((h.shape[0], m.heads * self.hv), dtype=h.dtype, device=h.device)
        if plan.expanded is not None:
            e = plan.expanded
            c = pages.view(-1, geo.rp + hr).index_select(0, e.ctx_slots)
            kv = self.ukv(c[:, :geo.rp])
            n = m.heads * geo.hd
            attention_ragged(q, kv[:, :n], kv[:, n:], e.items, m.heads, geo.hd, m.scale, a, gate=gate, each=m.gate_each,
                             window=m.window, kr=c[:, geo.rp:] if hr else None, rotary=self.rotary, pos=b.pos)
            T.op(f"L{self.layer} expanded attention")
        if plan.absorbed is not None:
            r = plan.absorbed
            ql = torch.empty((r.nt, m.heads * (geo.rp + hr)), dtype=h.dtype, device=h.device)
            head_proj(q, self.ukt, r.nt, ql, rows_in=r.rows, hr=hr, rotary=self.rotary, pos=r.tok_pos)
            ol = latent_attention(ql, pages, r, m.heads, m.scale, hr, m.window)
            head_proj(ol, self.uv, r.nt, a, rows_out=r.rows, gate=gate, each=m.gate_each)
            T.op(f"L{self.layer} latent attention")
        return self.o(a)


class DeltaMixer:
    def __init__(self, model, i: int, m: DeltaSpec, w: Weights):
        p = f"l{i}.mix."
        cfg = model.cfg
        self.layer, self.eps, self.shape = i, cfg.eps, delta_shape(m)
        win, offs = w.stack([p + n for n in ("q", "k", "v", "b", "a1", "g1")], model.wp)
        self.win = w.proj(win)
        self.offs, self.oa, self.og = tuple(offs[:4]), offs[4], offs[5]
        self.ra, self.rg = pad64(w.w[p + "a1"].shape[0]), pad64(w.w[p + "g1"].shape[0])
        hk, hv = m.heads * m.dim, m.heads * m.vdim
        self.a2 = w.proj(w.mat(p + "a2", pad64(hk), self.ra))
        self.g2 = w.proj(w.mat(p + "g2", pad64(hv), self.rg))
        self.cw = torch.cat([w.f32(f"{p}{n}.conv") for n in "qkv"]).T.contiguous()
        self.a_log, self.dt_bias, self.norm = w.f32(p + "A_log"), w.f32(p + "dt_bias"), w.f32(p + "norm")
        self.ld = padk(hv)
        self.o = w.proj(w.mat(p + "o", model.wp, self.ld))

    def __call__(self, model, h: torch.Tensor, b: Batch) -> torch.Tensor:
        z = self.win(h)
        a2 = self.a2(z[:, self.oa:self.oa + self.ra])
        g2 = self.g2(z[:, self.og:self.og + self.rg])
        T.op(f"L{self.layer} delta projections")
        o = delta_forward(z, self.offs, a2, self.cw, self.a_log, self.dt_bias, self.shape, model.state[self.layer],
                          b.seqs)
        y = delta_out(o, self.norm, g2, self.eps, self.ld)
        T.op(f"L{self.layer} delta rule")
        return self.o(y)


class DenseFF:
    def __init__(self, model, i: int, ff: int, w: Weights):
        p = f"l{i}.mlp."
        self.layer = i
        fp = padk(ff)
        self.gate_up = w.proj(torch.cat([w.mat(p + n, fp, model.wp) for n in ("gate", "up")]), gated="gelu_tanh")
        self.down = w.proj(w.mat(p + "down", model.wp, fp))

    def __call__(self, model, h: torch.Tensor, b: Batch) -> torch.Tensor:
        y = self.down(self.gate_up(h))
        T.op(f"L{self.layer} feed-forward")
        return y


# ------------------------------------------------------------------------ model
class HybridModel(RaggedModel):
    def __init__(self, cfg: RuruzenConfig, device="cuda", dtype: str = "bfloat16", seed: int = 0,
                 num_pages: int = 1024, state_slots: int = 256, weights: dict | None = None,
                 packed_decode: bool = True):
        if cfg.streams > MAX_STREAMS:
            raise ValueError(f"streams {cfg.streams} is above {MAX_STREAMS}")
        super().__init__()
        self.cfg, self.device, self.dtype = cfg, torch.device(device), DTYPES[dtype]
        self.has_state = self.delta_chunks = cfg.has_state
        self.wp = padk(cfg.width)
        raw = weights if weights is not None else cfg.load_weights(seed, self.device)
        w = Weights(raw, self.device, self.dtype, packed_decode)
        if self.dtype == torch.bfloat16:
            D.reserve_workspace(self.device)  # split-K partials, before any hipGraph capture
        self.head = w.proj(w.mat("embed", pad64(cfg.vocab), self.wp))
        self.embed = self.head.w
        self.embed_norm = w.f32("embed.norm")
        one = torch.ones(cfg.streams, dtype=torch.float32, device=self.device)
        self.subs = []    # (sublayer, layer, last of its layer, write-back mix, write-back out)
        self.inputs = []  # (read-out, norm weight) in front of each sublayer, then in front of the output
        for i, layer in enumerate(cfg.layers):
            mk = LatentMixer if isinstance(layer.mixer, LatentSpec) else DeltaMixer
            parts = [mk(self, i, layer.mixer, w)]
            if layer.ff is not None:
                parts.append(DenseFF(self, i, layer.ff, w))
            for q, part in enumerate(parts, 1):
                hc = f"l{i}.hc{q}."
                self.inputs.append((w.f32(hc + "in"), w.f32(f"l{i}.norm{q}")))
                self.subs.append((part, i, q == len(parts), w.f32(hc + "mix"), w.f32(hc + "out")))
        self.inputs.append((one, w.f32("final.norm")))
        self.geometries = {s[0].geo for s in self.subs if isinstance(s[0], LatentMixer)}
        self.cache = LatentCache(latent_sizes(cfg), num_pages, self.dtype, self.device)
        # slot 0 is the null slot of padded decode rows
        self.state = {i: DeltaState(delta_shape(x.mixer), state_slots + 1, self.device)
                      for i, x in enumerate(cfg.layers) if isinstance(x.mixer, DeltaSpec)}

    @classmethod
    def for_engine(cls, cfg: RuruzenConfig, ec, device, backend: str, num_pages: int) -> "HybridModel":
        cls.check_engine(ec, backend)
        if ec.prefix_caching and cfg.has_state:
            raise ValueError("prefix caching shares cache pages, not recurrent state: off for this model")
        return cls(cfg, device=device, dtype=ec.dtype, seed=ec.seed, num_pages=num_pages, state_slots=ec.max_batch,
                   packed_decode=ec.packed_decode)

    @staticmethod
    def memory(cfg: RuruzenConfig, dtype: str, slots: int) -> dict:
        """Bytes of the weights, of all state slots and of one page (engine sizing)."""
        from kgs.models.ruruzen import tensor_shapes

        size = DTYPES[dtype].itemsize
        n = sum(int(np.prod(s)) for s in tensor_shapes(cfg).values())
        state = sum(DeltaState.bytes_per_slot(delta_shape(x.mixer)) for x in cfg.layers
                    if isinstance(x.mixer, DeltaSpec))
        return {"weights": 3 * size * n, "state": (slots + 1) * state,
                "page": LatentCache.bytes_per_page(latent_sizes(cfg), size) or 1}

    def weight_bytes(self) -> int:
        from kgs.models.ruruzen import tensor_shapes

        return self.dtype.itemsize * sum(int(np.prod(s)) for s in tensor_shapes(self.cfg).values())

    # ------------------------------------------------------------------ forward
    @torch.no_grad()
    def forward(self, b: Batch) -> torch.Tensor:
        """Runs the batch; fp32 logits ``[rows wanted, vocab]``."""
        cfg = self.cfg
        x, h = hyper_embed(b.tokens, self.embed, self.embed_norm, *self.inputs[0], cfg.width, cfg.eps, ld=self.wp)
        for j, (sub, layer, last, mix, out) in enumerate(self.subs):
            y = sub(self, h, b)
            h = hyper_step(x, y, mix, out, *self.inputs[j + 1], cfg.eps, ld=self.wp)
            T.op(f"L{layer} streams")
            if last and self.on_layer is not None:
                self.on_layer(layer, x.sum(1))
        if b.logit_rows is not None:
            if b.logit_rows.shape[0] == 0:
                return torch.empty((0, cfg.vocab), dtype=torch.float32, device=self.device)
            h = h.index_select(0, b.logit_rows)
        logits = softcap(self.head(h), cfg.vocab, cfg.logit_softcap)
        T.op("logits")
        return logits
