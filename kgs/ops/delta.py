"""Gated delta rule with per-channel decay (``native/kernels/delta.hip``): short
convolutions, unit norms and decays, the recurrence over ragged portions of any
length (one token per sequence in decode), and the normed, gated output. The
recurrence and everything that enters it are fp32."""
from __future__ import annotations

import ctypes
from dataclasses import dataclass

import numpy as np
import torch

from . import _lib
from .hyper import _act, _f32

MAX_DIM = 256
CHUNK = 16       # tokens per chunk of the chunked form (delta.hip CH)
CHUNK_MIN = 16   # portions from here on go by chunks, shorter ones step token by token


@dataclass
class DeltaShape:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int

    def __post_init__(self):
        if self.dim > MAX_DIM:
            raise ValueError(f"delta-rule key size {self.dim} is above {MAX_DIM}")

    @property
    def kp(self) -> int:
        return (self.dim + 31) // 32 * 32

    @property
    def channels(self) -> int:
        return 2 * self.kv_heads * self.dim + self.heads * self.vdim


class DeltaState:
    """Per-slot state of one layer: ``S`` fp32 ``[slots, H, V, KP]`` (transposed,
    keys padded) and the convolution tails fp32 ``[slots, taps - 1, channels]``.
    A portion at position 0 ignores what its slot holds."""

    def __init__(self, shape: DeltaShape, slots: int, device):
        self.S = torch.zeros((slots, shape.heads, shape.vdim, shape.kp), dtype=torch.float32, device=device)
        self.conv = torch.zeros((slots, max(1, shape.taps - 1), shape.channels), dtype=torch.float32, device=device)

    @staticmethod
    def bytes_per_slot(shape: DeltaShape) -> int:
        return 4 * (shape.heads * shape.vdim * shape.kp + max(1, shape.taps - 1) * shape.channels)


@dataclass
class RaggedSeqs:
    """Sequences of a call (int32, device): each row's sequence, and per sequence
    its first row, rows, first position and state slot. ``chunks`` / ``cseqs`` (see
    :func:`chunk_plan`): the sequences that go by chunks; ``step_rows`` /
    ``step_seqs``: rows and numbers of the others, None when that is all of them."""
    row_seq: torch.Tensor
    row0: torch.Tensor
    n: torch.Tensor
    pos0: torch.Tensor
    slot: torch.Tensor
    chunks: torch.Tensor | None = None
    cseqs: torch.Tensor | None = None
    step_rows: torch.Tensor | None = None
    step_seqs: torch.Tensor | None = None


def chunk_plan(row0, n, pos0, slot) -> dict:
    """Host arrays of a batch's split: ``chunks [c, 8]`` (first row, rows, sequence, 0,
    then its sequence's first row, first position and state slot, 0), ``cseqs [s, 4]`` (sequence, first chunk, chunks, first row; longest first),
    ``step_rows``, ``step_seqs``. Empty when every sequence steps."""
    row0, n, pos0, slot = (np.asarray(x) for x in (row0, n, pos0, slot))
    big = np.flatnonzero(n >= CHUNK_MIN)
    if not len(big):
        return {}
    nc = -(-n[big] // CHUNK)
    first = np.cumsum(nc) - nc
    seq = np.repeat(big, nc)
    at = (np.arange(nc.sum()) - np.repeat(first, nc)) * CHUNK
    zero = np.zeros_like(seq)
    chunks = np.stack([row0[seq] + at, np.minimum(CHUNK, n[seq] - at), seq, zero, row0[seq], pos0[seq], slot[seq], zero],
                      1)
    cseqs = np.stack([big, first, nc, row0[big]], 1)[np.argsort(-nc, kind="stable")]
    small = np.flatnonzero(n < CHUNK_MIN)
    rows = np.concatenate([np.arange(row0[s], row0[s] + n[s]) for s in small]) if len(small) else np.zeros(0, np.int64)
    return {"chunks": chunks, "cseqs": cseqs, "step_rows": rows, "step_seqs": small}


def delta_forward(z: torch.Tensor, offs: tuple[int, int, int, int], a2: torch.Tensor, cw: torch.Tensor,
                  a_log: torch.Tensor, dt_bias: torch.Tensor, sh: DeltaShape, state: DeltaState,
                  seqs: RaggedSeqs) -> torch.Tensor:
    """The mixer up to its read-out: ``z`` the fused input projection with q, k, v
    and step-size columns at ``offs``, ``a2 [T, >= H * dim]`` the decay projection,
    ``cw [taps, channels]`` the convolutions. Returns o fp32 ``[T, H, V]``; the
    sequences' states and convolution tails are advanced in place."""
    T, dev = z.shape[0], z.device
    H, G, K, V = sh.heads, sh.kv_heads, sh.dim, sh.vdim
    _act(z, T, max(offs[0] + G * K, offs[1] + G * K, offs[2] + H * V, offs[3] + H), z.dtype, "z")
    _act(a2, T, H * K, z.dtype, "a2")
    B = seqs.row0.shape[0]

    def f32(*shape):
        return torch.empty(shape, dtype=torch.float32, device=dev)

    o = f32(T, H, V)
    nc = 0 if seqs.chunks is None else seqs.chunks.shape[0]
    nstep = (T, B) if not nc else (seqs.step_rows.shape[0], seqs.step_seqs.shape[0])
    # indexed by row: only stepped rows' parts are touched
    prep = [f32(T, G, sh.kp), f32(T, G, sh.kp), f32(T, H, V), f32(T, H, sh.kp), f32(T, H), f32(T, G)] if nstep[0] else []
    work = [f32(nc, H, CHUNK, sh.kp), f32(nc, H, CHUNK, sh.kp), f32(nc, H, sh.kp, CHUNK), f32(nc, H, sh.kp),
            f32(nc, H, CHUNK, V), f32(nc, H, CHUNK, CHUNK)] if nc else []
    ptr = lambda ts, n: [t.data_ptr() for t in ts] if ts else [0] * n  # noqa: E731
    opt = lambda t: 0 if t is None or not nc else t.data_ptr()  # noqa: E731
    ptrs = (ctypes.c_void_p * 29)(
        z.data_ptr(), a2.data_ptr(), _f32(cw, (sh.taps, sh.channels), "cw"), _f32(a_log, (H,), "a_log"),
        _f32(dt_bias, (H * K,), "dt_bias"), seqs.row_seq.data_ptr(), seqs.row0.data_ptr(), seqs.n.data_ptr(),
        seqs.pos0.data_ptr(), seqs.slot.data_ptr(), *ptr(prep, 6), o.data_ptr(), state.S.data_ptr(),
        state.conv.data_ptr(), opt(seqs.step_rows), opt(seqs.step_seqs), opt(seqs.chunks), opt(seqs.cseqs), *ptr(work, 6))
    pairs = not (K % 2 or V % 2 or z.stride(0) % 2 or a2.stride(0) % 2 or any(x % 2 for x in offs[:3]) or
                 z.data_ptr() % 4 or a2.data_ptr() % 4)
    dims = (ctypes.c_long * 20)(z.stride(0), a2.stride(0), *offs, sh.taps, G, H, K, V, sh.kp, B, T,
                                int(z.dtype == torch.float32), *nstep, nc, seqs.cseqs.shape[0] if nc else 0, int(pairs))
    _lib.check(_lib.lib().kgs_delta_forward(ptrs, dims, _lib.stream_handle(dev)), f"delta_forward[{T}x{H}x{K}x{V}]")
    return o


def delta_out(o: torch.Tensor, w: torch.Tensor, gate: torch.Tensor, eps: float, ld: int) -> torch.Tensor:
    """``rmsnorm(o) * w * sigmoid(gate)`` per head -> ``[T, ld]`` in the gate's
    dtype (zero past ``H * V``)."""
    T, H, V = o.shape
    y = torch.empty((T, ld), dtype=gate.dtype, device=o.device)
    rc = _lib.lib().kgs_delta_out(_f32(o, (T, H, V), "o"), _f32(w, (V,), "w"), _act(gate, T, H * V, gate.dtype, "gate"),
                                  y.data_ptr(), T, H, V, gate.stride(0), ld, float(eps),
                                  int(gate.dtype == torch.float32), _lib.stream_handle(o.device))
    _lib.check(rc, f"delta_out[{T}x{H}x{V}]")
    return y
