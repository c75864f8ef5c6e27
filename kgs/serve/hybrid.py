"""Serving model of layer stacks that mix latent attention and delta-rule mixers
over hyper-connected residual streams (:mod:`kgs.models.ruruzen`).

Every step -- prompts, prompt portions, mixed steps, decode -- is one ragged batch
(:class:`Batch`): each sequence brings some tokens at some position, reads and
extends its latent pages, and advances its recurrent state in its slot. The
same :meth:`HybridModel.forward` runs all of them; decode steps (one token per
sequence) have fixed shapes and are captured in hipGraphs by the engine.

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
from kgs.ops.delta import DeltaShape, DeltaState, RaggedSeqs, chunk_plan, delta_forward, delta_out
from kgs.ops.hyper import MAX_STREAMS, hyper_embed, hyper_step
from kgs.ops.latent import (KERNEL_SIZES, LatentCache, LatentRows, head_proj, latent_attention, latent_norm,
                            padded_latent, split_count, waves_for)
from kgs.ops.linear import Projection
from kgs.ops.transformer import attention_ragged

from .trace import TRACE as T

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}
EXPAND_MIN = 16  # shorter portions are not worth the expansion's launches
QBLOCK = 128  # query rows of one attention_ragged item


def pad64(n: int) -> int:
    return (n + 63) // 64 * 64


def padk(n: int) -> int:
    """Padded size of a GEMM's inner dimension: the MFMA GEMMs step by 128, which a
    small one is not padded to."""
    return pad64(n) if n <= 512 else (n + 127) // 128 * 128


def _pad(w: torch.Tensor, *sizes: int) -> torch.Tensor:
    """``w`` zero-padded at the end of its last ``len(sizes)`` dimensions."""
    pads = []
    for d, s in zip(reversed(w.shape), reversed(sizes)):
        pads += [0, s - d]
    return torch.nn.functional.pad(w, pads)


def latent_sizes(cfg: RuruzenConfig) -> dict[int, int]:
    """Padded latent size of every layer that caches one."""
    return {i: padded_latent(x.mixer.kv_rank) for i, x in enumerate(cfg.layers)
            if isinstance(x.mixer, LatentSpec) and x.mixer.kv_from is None}


def delta_shape(m: DeltaSpec) -> DeltaShape:
    return DeltaShape(m.heads, m.kv_heads, m.dim, m.vdim, m.conv)


# --------------------------------------------------------------------- batches
class HostPack:
    """int32 arrays of one step, sent to the device in one copy."""

    def __init__(self, device):
        self.device, self.parts, self.size = device, [], 0

    def add(self, a) -> tuple[int, tuple]:
        a = np.ascontiguousarray(a, dtype=np.int32)
        ref = (self.size, a.shape)
        self.parts.append(a.reshape(-1))
        pad = -a.size % 4  # every array 16-B aligned
        if pad:
            self.parts.append(np.zeros(pad, np.int32))
        self.size += a.size + pad
        return ref

    def send(self):
        t = torch.from_numpy(np.concatenate(self.parts) if self.parts else np.zeros(4, np.int32))
        if self.device.type == "cuda":
            t = t.pin_memory().to(self.device, non_blocking=True)
        return lambda ref: t[ref[0]:ref[0] + int(np.prod(ref[1]))].view(ref[1])


@dataclass
class Expanded:
    """Portions that attend over expanded keys and values."""
    items: torch.Tensor        # attention_ragged items
    ctx_slots: torch.Tensor    # cache slot of every key, the sequences one after another (int64)


@dataclass
class LatentPlan:
    absorbed: LatentRows | None
    expanded: Expanded | None


@dataclass
class Batch:
    tokens: torch.Tensor       # [T] int32
    slots: torch.Tensor        # [T] cache slot of each row, -1: none
    seqs: RaggedSeqs
    plans: dict                # latent geometry -> LatentPlan
    logit_rows: torch.Tensor | None  # rows whose logits are wanted (None: every row)


@dataclass(frozen=True)
class Geometry:
    """What a latent-attention launch plan depends on."""
    heads: int
    rp: int
    hd: int                    # head size of the expanded form, 0: absorbed only

    def expand(self, n: int, pos0: int) -> bool:
        """Whether a portion of ``n`` tokens after ``pos0`` runs on expanded keys and
        values. Per head that expands every context token (``4 rp hd`` flops each)
        where the absorbed form maps every query token (as many), and pays ``4 hd``
        per (query, key) pair where the absorbed form pays ``4 rp``."""
        pairs = n * (pos0 + 0.5 * n)
        return self.hd > 0 and n >= EXPAND_MIN and pos0 * self.rp * self.hd < (self.rp - self.hd) * pairs


# -------------------------------------------------------------------- sublayers
class _Weights:
    """Checkpoint tensors on their way to the device layout."""

    def __init__(self, w: dict, device, dtype, pack: bool):
        self.w, self.device, self.dtype, self.pack = w, device, dtype, pack

    def proj(self, t: torch.Tensor, gated: str | None = None) -> Projection:
        return Projection(t, gated, pack=self.pack)

    def f32(self, name: str) -> torch.Tensor:
        return self.w[name].to(self.device).float().contiguous()

    def mat(self, name: str, rows: int, cols: int) -> torch.Tensor:
        return _pad(self.w[name].to(self.device).to(self.dtype), rows, cols)

    def stack(self, names, cols: int) -> tuple[torch.Tensor, list[int]]:
        """Several projections of one input as one matrix, each from a multiple of
        64 rows on (a large one ends on whole GEMM tiles); returns it and the first rows."""
        parts, offs, n = [], [], 0
        for name in names:
            p = self.mat(name, pad64(self.w[name].shape[0]), cols)
            offs.append(n)
            n += p.shape[0]
            parts.append(p)
        if n > 1024 and n % 256:  # whole 256-wide GEMM tiles
            parts.append(torch.zeros((256 - n % 256, cols), dtype=self.dtype, device=self.device))
        return torch.cat(parts).contiguous(), offs


class LatentMixer:
    def __init__(self, model, i: int, m: LatentSpec, w: _Weights):
        p = f"l{i}.mix."
        cfg = model.cfg
        self.m, self.owner = m, i if m.kv_from is None else m.kv_from
        self.layer = i
        self.eps = cfg.eps
        names = ["dq", "g"] + (["dkv"] if m.kv_from is None else [])
        win, offs = w.stack([p + n for n in names], model.wp)
        self.win = w.proj(win)
        self.oq, self.og = offs[0], offs[1]
        self.oc = offs[2] if m.kv_from is None else 0
        self.wq = w.f32(p + "dq.norm")
        self.wc = w.f32(p + "dkv.norm") if m.kv_from is None else None
        self.qp = padk(m.q_rank)
        rp = padded_latent(m.kv_rank)
        both = max(m.dim, m.vdim)
        hd = (64 if both <= 64 else 128 if both <= 128 else 0) if w.dtype == torch.bfloat16 else 0
        self.hq, self.hv = (hd, hd) if hd else (pad64(m.dim), pad64(m.vdim))
        self.geo = Geometry(m.heads, rp, hd)
        H = m.heads

        def heads(name, d, dp, rank, rankp):
            t = w.w[p + name].to(w.device).to(w.dtype).reshape(H, d, rank)
            return _pad(t, dp, rankp)

        self.uq = w.proj(heads("uq", m.dim, self.hq, m.q_rank, self.qp).reshape(H * self.hq, self.qp))
        uk = heads("uk", m.dim, self.hq, m.kv_rank, rp)
        self.uv = heads("uv", m.vdim, self.hv, m.kv_rank, rp).contiguous()          # [H, HV, RP]
        self.ukt = uk.transpose(1, 2).contiguous()                                  # [H, RP, HQ]
        self.ukv = Projection(torch.cat([uk.reshape(-1, rp), self.uv.reshape(-1, rp)]), pack=False) if hd else None
        o = w.w[p + "o"].to(w.device).to(w.dtype).reshape(cfg.width, H, m.vdim)
        self.o = w.proj(_pad(_pad(o, self.hv).reshape(cfg.width, H * self.hv), model.wp, H * self.hv))

    def __call__(self, model, h: torch.Tensor, b: Batch) -> torch.Tensor:
        m, geo = self.m, self.geo
        z = self.win(h)
        pages = model.cache.pages[self.owner]
        cq = latent_norm(z, self.oq, self.wq, self.qp, self.oc, self.wc, pages if self.wc is not None else None,
                         b.slots, self.eps)
        q = self.uq(cq)
        T.op(f"L{self.layer} latent projections")
        gate = z[:, self.og:self.og + m.heads]
        plan = b.plans[geo]
        a = torch.empty((h.shape[0], m.heads * self.hv), dtype=h.dtype, device=h.device)
        if plan.expanded is not None:
            e = plan.expanded
            c = pages.view(-1, geo.rp).index_select(0, e.ctx_slots)
            kv = self.ukv(c)
            n = m.heads * geo.hd
            attention_ragged(q, kv[:, :n], kv[:, n:], e.items, m.heads, geo.hd, m.scale, a, gate=gate)
            T.op(f"L{self.layer} expanded attention")
        if plan.absorbed is not None:
            r = plan.absorbed
            ql = torch.empty((r.nt, m.heads * geo.rp), dtype=h.dtype, device=h.device)
            head_proj(q, self.ukt, r.nt, ql, rows_in=r.rows)
            ol = latent_attention(ql, pages, r, m.heads, m.scale)
            head_proj(ol, self.uv, r.nt, a, rows_out=r.rows, gate=gate)
            T.op(f"L{self.layer} latent attention")
        return self.o(a)


class DeltaMixer:
    def __init__(self, model, i: int, m: DeltaSpec, w: _Weights):
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
    def __init__(self, model, i: int, ff: int, w: _Weights):
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
class HybridModel:
    """Serving interface: ``ragged`` (steps come as plans, :meth:`run_plan`, decode
    as fixed-shape device tensors, :meth:`decode`), ``has_state`` (the scheduler
    hands out a state slot per running sequence)."""

    DTYPES = tuple(DTYPES)
    ragged = True
    pad_multiple = 1  # portions are not padded

    def __init__(self, cfg: RuruzenConfig, device="cuda", dtype: str = "bfloat16", seed: int = 0,
                 num_pages: int = 1024, state_slots: int = 256, weights: dict | None = None,
                 packed_decode: bool = True):
        if cfg.streams > MAX_STREAMS:
            raise ValueError(f"streams {cfg.streams} is above {MAX_STREAMS}")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), DTYPES[dtype]
        self.has_state = cfg.has_state
        self.wp = padk(cfg.width)
        raw = weights if weights is not None else cfg.load_weights(seed, self.device)
        w = _Weights(raw, self.device, self.dtype, packed_decode)
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
        self._fixed: dict = {}
        self.on_layer = None  # tests: called with (layer, sum of the streams) after every layer

    @classmethod
    def for_engine(cls, cfg: RuruzenConfig, ec, device, backend: str, num_pages: int) -> "HybridModel":
        if backend != "kgs":
            raise ValueError("this model runs on the GPU kernels only (backend 'kgs')")
        for name in ("decode_weights", "kv_cache_dtype", "prefill_weights"):
            if getattr(ec, name) != "bf16":
                raise ValueError(f"{name}={getattr(ec, name)!r} is not available for this model")
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

    # -------------------------------------------------------------------- plans
    def run_plan(self, plan, tokens: torch.Tensor | None = None, logit_rows=None) -> torch.Tensor:
        """A prefill or mixed plan. ``tokens``: the input tokens on the device when
        some are still being sampled. ``logit_rows``: the rows wanted (default: each
        prompt's last row where its portion ends it, then the decode rows)."""
        npf, T_ = plan.n_prefill, len(plan.tokens)
        nd = len(plan.seq_ids) - npf
        lens, starts = np.asarray(plan.seq_lens), np.asarray(plan.seq_starts)
        row0 = np.concatenate([starts, np.arange(T_ - nd, T_)]).astype(np.int64)
        n = np.concatenate([lens, np.ones(nd, np.int64)]).astype(np.int64)
        pos0 = np.concatenate([np.asarray(plan.ctx_starts), np.asarray(plan.ctx_lens) - 1]).astype(np.int64)
        slot = np.asarray(plan.state_slots) if self.has_state else np.zeros(len(n), np.int64)
        W = max(1, plan.pf_max_pages, plan.max_pages)
        bt = np.zeros((len(n), W), np.int32)
        if npf:
            bt[:npf, :plan.pf_max_pages] = plan.pf_block_tables
        if nd:
            bt[npf:, :plan.max_pages] = plan.block_tables
        if logit_rows is None:
            last = np.asarray(plan.last_chunk).astype(bool)
            logit_rows = np.concatenate([(starts + lens - 1)[last], np.arange(T_ - nd, T_)])
        return self.forward(self.batch(np.asarray(plan.tokens), np.asarray(plan.slots), row0, n, pos0, slot, bt,
                                       logit_rows, tokens))

    def batch(self, tokens, slots, row0, n, pos0, slot, bt, logit_rows, dev_tokens=None) -> Batch:
        """A ragged batch from host arrays; one host-to-device copy."""
        pk = HostPack(self.device)
        row_seq = np.repeat(np.arange(len(n)), n)
        order = np.argsort(row0, kind="stable")  # rows of the batch are the sequences' rows in row0 order
        if len(row_seq) != len(tokens) or not np.array_equal(np.cumsum(n[order]) - n[order], row0[order]):
            raise ValueError("the sequences' rows do not tile the batch")
        row_seq = np.repeat(order, n[order])
        pos = pos0[row_seq] + np.arange(len(tokens)) - row0[row_seq]
        refs = [pk.add(a) for a in (tokens, slots, row_seq, row0, n, pos0, slot, bt, logit_rows)]
        split = {k: pk.add(v) for k, v in chunk_plan(row0, n, pos0, slot).items()} if self.has_state else {}
        host = {g: self._host_plan(pk, g, row0, n, pos0, bt, row_seq, pos, refs) for g in self.geometries}
        get = pk.send()
        d = [get(r) for r in refs]
        plans = {}
        for g, (a, e) in host.items():
            absorbed = None
            if a is not None:
                r, shape = a
                dev = {k: (None if v is None else get(v)) for k, v in r.items()}
                absorbed = LatentRows(**dev, **shape)
            expanded = None if e is None else Expanded(get(e[0]), get(e[1]).long())
            plans[g] = LatentPlan(absorbed, expanded)
        return Batch(dev_tokens.to(torch.int32).contiguous() if dev_tokens is not None else d[0], d[1],
                     RaggedSeqs(d[2], d[3], d[4], d[5], d[6], **{k: get(r) for k, r in split.items()}), plans, d[8].long())

    @staticmethod
    def _host_plan(pk: HostPack, g: Geometry, row0, n, pos0, bt, row_seq, pos, refs):
        """Splits the sequences between the absorbed and the expanded form and lays
        out both launches; returns references into ``pk``."""
        big = np.array([g.expand(int(x), int(p)) for x, p in zip(n, pos0)], bool)
        absorbed = expanded = None
        sel = np.flatnonzero(~big)
        if len(sel):
            ns = n[sel]
            q0 = np.cumsum(ns) - ns
            rows = ns * g.heads
            waves = waves_for(int(rows.max()), g.rp)
            tiles = -(-rows // (16 * waves))
            # the tiles with the longest context first
            seq = np.repeat(np.arange(len(sel)), tiles)
            tile = np.arange(len(seq)) - np.repeat(np.cumsum(tiles) - tiles, tiles)
            end = pos0[sel][seq] + np.minimum((tile + 1) * 16 * waves, rows[seq]) // g.heads
            o = np.argsort(-end, kind="stable")
            items = np.stack([seq[o], tile[o]], 1)
            ident = len(sel) == len(n) and np.array_equal(q0, row0)
            order = None if ident else np.concatenate([np.arange(r, r + c) for r, c in zip(row0[sel], ns)])
            at = np.arange(len(row_seq)) if order is None else order
            maxp = int((pos0[sel] + ns - 1).max()) // PAGE + 1
            absorbed = ({"q0": pk.add(q0), "n": pk.add(ns), "pos0": pk.add(pos0[sel]),
                         "bt": refs[7] if ident else pk.add(bt[sel]),
                         "tok_seq": pk.add(np.repeat(np.arange(len(sel)), ns)), "tok_pos": pk.add(pos[at]),
                         "rows": None if order is None else pk.add(order), "items": pk.add(items)},
                        {"nt": int(ns.sum()), "ntiles": len(items), "tiles": 0, "waves": waves,
                         "nsplit": split_count(len(items), maxp, g.rp)})
        sel = np.flatnonzero(big)
        if len(sel):
            items, ctx, base = [], [], 0
            for s in sel:
                total = int(pos0[s] + n[s])
                p = np.arange(total)
                ctx.append(bt[s][p // PAGE].astype(np.int64) * PAGE + p % PAGE)
                for q in range(0, int(n[s]), QBLOCK):
                    items.append((row0[s] + q, base, pos0[s] + q, min(QBLOCK, n[s] - q)))
                base += total
            items = np.array(items, np.int64)
            items = items[np.argsort(-(items[:, 2] + items[:, 3]), kind="stable")]
            expanded = (pk.add(items), pk.add(np.concatenate(ctx)))
        return absorbed, expanded

    # ------------------------------------------------------------------- decode
    def _fixed_seqs(self, nb: int) -> dict:
        """Index tensors of a decode batch of ``nb`` sequences, one row each."""
        if nb not in self._fixed:
            ar = torch.arange(nb, dtype=torch.int32, device=self.device)
            self._fixed[nb] = {"ar": ar, "one": torch.ones_like(ar), "zero": torch.zeros_like(ar)}
        return self._fixed[nb]

    def decode(self, tokens, positions, slots, block_tables, ctx_lens, state_slots=None) -> torch.Tensor:
        """One token per sequence, everything on the device (hipGraph capture)."""
        nb, W = block_tables.shape
        f = self._fixed_seqs(nb)
        plans = {}
        for g in self.geometries:
            waves = waves_for(g.heads, g.rp)
            tiles = -(-g.heads // (16 * waves))
            plans[g] = LatentPlan(LatentRows(
                nt=nb, q0=f["ar"], n=f["one"], pos0=positions, bt=block_tables, tok_seq=f["ar"], tok_pos=positions,
                rows=None, items=None, ntiles=nb * tiles, tiles=tiles, waves=waves,
                nsplit=split_count(nb * tiles, W, g.rp)), None)
        seqs = RaggedSeqs(f["ar"], f["ar"], f["one"], positions, state_slots if self.has_state else f["zero"])
        return self.forward(Batch(tokens, slots, seqs, plans, None))
