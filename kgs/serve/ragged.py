"""What the ragged serving models share: every step -- prompts, prompt portions,
mixed steps, decode -- is one :class:`Batch`; each sequence brings some tokens at
some position, reads and extends its cache pages, and advances its recurrent state
(where the model has one) in its slot. :class:`RaggedModel` turns scheduler plans
and fixed-shape decode steps into batches for a model's ``forward``.

A model's attention layers of equal shape share a *geometry*: a hashable object that
lays out their launches once per step, from host arrays (``host_plan``) or for a
decode step on the device (``decode_plan``).

:class:`Weights` lays a checkpoint out on the device: projections of one input fused
into one matrix, every dimension that a GEMM sees padded with zeros.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from kgs.ops.delta import RaggedSeqs, chunk_plan
from kgs.ops.linear import Projection
from kgs.ops.talking import Rotary

DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}


def pad64(n: int) -> int:
    return (n + 63) // 64 * 64


def pad128(n: int) -> int:
    return (n + 127) // 128 * 128


def pad256(n: int) -> int:
    return (n + 255) // 256 * 256


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
class Batch:
    tokens: torch.Tensor       # [T] int32
    slots: torch.Tensor        # [T] cache slot of each row, -1: none
    seqs: RaggedSeqs
    plans: dict                # attention geometry -> its launch plan
    logit_rows: torch.Tensor | None  # rows whose logits are wanted (None: every row)
    pos: torch.Tensor | None = None  # [T] int32 position of each row


# --------------------------------------------------------------------- weights
class Weights:
    """Checkpoint tensors on their way to the device layout."""

    def __init__(self, w: dict, device, dtype, pack: bool):
        self.w, self.device, self.dtype, self.pack = w, device, dtype, pack

    def proj(self, t: torch.Tensor, gated=None) -> Projection:
        return Projection(t, gated, pack=self.pack)

    def f32(self, name: str) -> torch.Tensor:
        return self.w[name].to(self.device).float().contiguous()

    def mat(self, name: str, rows: int, cols: int) -> torch.Tensor:
        return _pad(self.w[name].to(self.device).to(self.dtype), rows, cols)

    def heads(self, t: torch.Tensor, n: int, d: int, dp: int) -> torch.Tensor:
        """``[n d, ..] -> [n dp, ..]`` on the device, every head padded."""
        t = t.to(self.device).to(self.dtype)
        return _pad(t.reshape(n, d, -1), dp, t.shape[-1]).reshape(n * dp, -1)

    def stack(self, names, cols: int) -> tuple[torch.Tensor, list[int]]:
        """Several projections of one input as one matrix, each from a multiple of
        64 rows on (a large one ends on whole GEMM tiles); returns it and the first rows."""
        return self.join([self.w[name] for name in names], cols)

    def join(self, tensors, cols: int) -> tuple[torch.Tensor, list[int]]:
        """:meth:`stack` of tensors."""
        parts, offs, n = [], [], 0
        for t in tensors:
            p = _pad(t.to(self.device).to(self.dtype), pad64(t.shape[0]), cols)
            offs.append(n)
            n += p.shape[0]
            parts.append(p)
        if n > 1024 and n % 256:  # whole 256-wide GEMM tiles
            parts.append(torch.zeros((256 - n % 256, cols), dtype=self.dtype, device=self.device))
        return torch.cat(parts).contiguous(), offs


# ------------------------------------------------------------------------ model
class RaggedModel:
    """Serving interface: ``ragged`` (steps come as plans, :meth:`run_plan`, decode
    as fixed-shape device tensors, :meth:`decode`), ``has_state`` (the scheduler
    hands out a state slot per running sequence). A model sets ``device``,
    ``has_state``, ``geometries`` and has ``forward(batch)``."""

    DTYPES = tuple(DTYPES)
    ragged = True
    pad_multiple = 1  # portions are not padded
    has_state = False
    delta_chunks = False  # batches carry the delta rule's split into chunks

    def __init__(self):
        self._fixed: dict = {}
        self.geometries: set = set()
        self.max_len, self._rotary = 0, {}  # positions of the rotary tables, and these
        self.on_layer = None  # tests: called with (layer, residual) after every layer

    def rotary(self, dims: int, base: float) -> Rotary:
        if (dims, base) not in self._rotary:
            self._rotary[dims, base] = Rotary(dims, base, self.max_len, self.device)
        return self._rotary[dims, base]

    @staticmethod
    def check_engine(ec, backend: str) -> None:
        """The engine options these models do not have."""
        if backend != "kgs":
            raise ValueError("this model runs on the GPU kernels only (backend 'kgs')")
        for name in ("decode_weights", "kv_cache_dtype", "prefill_weights"):
            if getattr(ec, name) != "bf16":
                raise ValueError(f"{name}={getattr(ec, name)!r} is not available for this model")

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
        refs = [pk.add(a) for a in (tokens, slots, row_seq, row0, n, pos0, slot, bt, logit_rows, pos)]
        split = {k: pk.add(v) for k, v in chunk_plan(row0, n, pos0, slot).items()} if self.delta_chunks else {}
        host = {g: g.host_plan(pk, row0, n, pos0, bt, row_seq, pos, refs) for g in self.geometries}
        get = pk.send()
        d = [get(r) for r in refs]
        plans = {g: build(get) for g, build in host.items()}
        return Batch(dev_tokens.to(torch.int32).contiguous() if dev_tokens is not None else d[0], d[1],
                     RaggedSeqs(d[2], d[3], d[4], d[5], d[6], **{k: get(r) for k, r in split.items()}), plans, d[8].long(),
                     d[9])

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
        plans = {g: g.decode_plan(f, nb, positions, block_tables) for g in self.geometries}
        seqs = RaggedSeqs(f["ar"], f["ar"], f["one"], positions, state_slots if self.has_state else f["zero"])
        return self.forward(Batch(tokens, slots, seqs, plans, None, positions))
