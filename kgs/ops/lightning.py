"""Lightning attention (``native/kernels/lightning.hip``): a linear recurrence with one
fixed decay per head over ragged portions of any length (one token per sequence in
decode), and the normed, gated output. The state and the recurrence are fp32.

Portions from :data:`CHUNK_MIN` tokens go by chunks on bf16 MFMAs (:func:`segment_plan`
cuts long ones into segments that run side by side), shorter ones and fp32 token by token.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from . import _lib
from .decode import CUS
from .delta import RaggedSeqs
from .hyper import _act, _f32

CHUNK = 64         # tokens of a chunk (lightning.hip C)
CHUNK_MIN = 16     # portions from here on go by chunks
MAX_SEGMENT = 64   # chunks of a segment
MAX_DIM = 256      # key size (by chunks: up to 128)
CHUNK_DIM = 128


@dataclass(frozen=True)
class LightningShape:
    heads: int
    dim: int
    vdim: int

    def __post_init__(self):
        if self.dim > MAX_DIM:
            raise ValueError(f"lightning key size {self.dim} is above {MAX_DIM}")

    @property
    def kp(self) -> int:
        return next(s for s in (64, 128, 256) if s >= self.dim)

    @property
    def vp(self) -> int:
        return 64 if self.vdim <= 64 else (self.vdim + 127) // 128 * 128

    @property
    def slabs(self) -> int:
        """Workgroups that share a head's value columns."""
        return max(1, self.vp // 128)


class LightningState:
    """One layer's states, fp32 ``[slots, H, KP, VP]``. A portion at position 0 ignores
    what its slot holds."""

    def __init__(self, shape: LightningShape, slots: int, device):
        self.S = torch.zeros((slots, shape.heads, shape.kp, shape.vp), dtype=torch.float32, device=device)

    @staticmethod
    def bytes_per_slot(shape: LightningShape) -> int:
        return 4 * shape.heads * shape.kp * shape.vp


class Decays:
    """Powers of the heads' decays: of one token (0 .. CHUNK) and of whole chunks."""

    def __init__(self, decay, device):
        d = torch.tensor(list(decay), dtype=torch.float64)[:, None]
        self.tokens = (d ** torch.arange(CHUNK + 1)).float().to(device).contiguous()
        self.chunks = ((d ** CHUNK) ** torch.arange(MAX_SEGMENT + 1)).float().to(device).contiguous()


@dataclass
class SegmentPlan:
    """``seqs``: the sequences that step (None: all ``nstep``); ``items``, ``scans``: see
    :func:`segment_plan` (None: none); ``buffers``: states between segments."""
    nstep: int
    seqs: torch.Tensor | None = None
    items: torch.Tensor | None = None
    scans: torch.Tensor | None = None
    buffers: int = 0


def segment_plan(n, units: int, chunked: bool = True) -> dict:
    """Host arrays of a batch's split, sequences of ``n`` tokens: ``step`` (sequences that
    go token by token), ``items [i, 4]`` (sequence, first token, tokens, buffer or -1;
    longest first) and ``scans [s, 4]`` (sequence, first buffer, segments, chunks of a
    full segment). ``units``: workgroups of one segment. A sequence is cut where the
    sequences alone leave CUs idle, into segments that fill them about twice."""
    n = np.asarray(n)
    big = np.flatnonzero((n >= CHUNK_MIN) & chunked)
    step = np.flatnonzero((n < CHUNK_MIN) | (not chunked))
    items, scans, nbuf = [], [], 0
    if len(big):
        chunks = -(-n[big] // CHUNK)
        seg = MAX_SEGMENT
        if len(big) * units < CUS:
            seg = min(MAX_SEGMENT, max(2, -(-int(chunks.sum()) * units // (2 * CUS))))
        for s, c in zip(big, chunks):
            ns = -(-int(c) // seg)
            starts = np.arange(ns) * seg * CHUNK
            buf = nbuf + np.arange(ns) if ns > 1 else np.array([-1])
            items.append(np.stack([np.full(ns, s), starts, np.minimum(seg * CHUNK, n[s] - starts), buf], 1))
            if ns > 1:
                scans.append((s, nbuf, ns, seg))
                nbuf += ns
        items = np.concatenate(items)
        items = items[np.argsort(-items[:, 2], kind="stable")]
    return {"step": step, "items": items, "scans": scans, "buffers": nbuf}


def lightning_forward(z: torch.Tensor, offs: tuple[int, int, int], sh: LightningShape, decays: Decays,
                      state: LightningState, seqs: RaggedSeqs, plan: SegmentPlan) -> torch.Tensor:
    """o fp32 ``[T, H * VP]`` before its norm: ``z`` the fused input projection with q, k
    and v columns at ``offs``, heads padded to KP / VP with zero columns. The sequences'
    states are advanced in place."""
    T, H, kp, vp = z.shape[0], sh.heads, sh.kp, sh.vp
    f32 = z.dtype == torch.float32
    _act(z, T, max(offs[0] + H * kp, offs[1] + H * kp, offs[2] + H * vp), z.dtype, "z")
    if state.S.shape[1:] != (H, kp, vp):
        raise ValueError(f"state {tuple(state.S.shape)} does not fit {sh}")
    ni = 0 if plan.items is None else plan.items.shape[0]
    nsc = 0 if plan.scans is None else plan.scans.shape[0]
    for t, c in ((plan.items, ni), (plan.scans, nsc)):
        if c and (t.dtype != torch.int32 or not t.is_contiguous() or t.shape[1] != 4):
            raise ValueError("items and scans must be contiguous int32 [n, 4]")
    o = torch.empty((T, H * vp), dtype=torch.float32, device=z.device)
    buf = torch.empty((plan.buffers, H, kp, vp), dtype=torch.float32, device=z.device) if plan.buffers else None
    opt = lambda t: 0 if t is None else t.data_ptr()  # noqa: E731
    rc = _lib.lib().kgs_lightning_forward(
        z.data_ptr(), z.stride(0), *offs, seqs.row0.data_ptr(), seqs.n.data_ptr(), seqs.pos0.data_ptr(),
        seqs.slot.data_ptr(), opt(plan.seqs), plan.nstep, opt(plan.items), ni, opt(plan.scans), nsc,
        _f32(decays.tokens, (H, CHUNK + 1), "decays"), _f32(decays.chunks, (H, MAX_SEGMENT + 1), "decays"), MAX_SEGMENT,
        state.S.data_ptr(), opt(buf), o.data_ptr(), H, kp, vp, int(f32), _lib.stream_handle(z.device))
    _lib.check(rc, f"lightning_forward[{T}x{H}x{kp}x{vp}]")
    return o


def lightning_out(o: torch.Tensor, w: torch.Tensor, gate: torch.Tensor, count: int, eps: float, ld: int) -> torch.Tensor:
    """``rmsnorm(o) * w * sigmoid(gate)`` over all heads together (``count`` columns that
    are not padding) -> ``[T, ld]`` in the gate's dtype, zero past the heads."""
    T, n = o.shape
    y = torch.empty((T, ld), dtype=gate.dtype, device=o.device)
    rc = _lib.lib().kgs_lightning_out(_f32(o, (T, n), "o"), _f32(w, (n,), "w"), _act(gate, T, n, gate.dtype, "gate"),
                                      gate.stride(0), y.data_ptr(), ld, T, n, count, float(eps),
                                      int(gate.dtype == torch.float32), _lib.stream_handle(o.device))
    _lib.check(rc, f"lightning_out[{T}x{n}]")
    return y
