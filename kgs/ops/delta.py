"""Gated delta rule with per-channel decay (``native/kernels/delta.hip``): short
convolutions, unit norms and decays, the recurrence over ragged portions of any
length (one token per sequence in decode), and the normed, gated output. The
recurrence and everything that enters it are fp32."""
from __future__ import annotations

import ctypes
from dataclasses import dataclass

import torch

from . import _lib
from .hyper import _act, _f32

MAX_DIM = 256


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
    its first row, rows, first position and state slot."""
    row_seq: torch.Tensor
    row0: torch.Tensor
    n: torch.Tensor
    pos0: torch.Tensor
    slot: torch.Tensor


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

    q, k, v, lg = f32(T, G, sh.kp), f32(T, G, sh.kp), f32(T, H, V), f32(T, H, sh.kp)
    beta, qk, o = f32(T, H), f32(T, G), f32(T, H, V)
    ptrs = (ctypes.c_void_p * 19)(
        z.data_ptr(), a2.data_ptr(), _f32(cw, (sh.taps, sh.channels), "cw"), _f32(a_log, (H,), "a_log"),
        _f32(dt_bias, (H * K,), "dt_bias"), seqs.row_seq.data_ptr(), seqs.row0.data_ptr(), seqs.n.data_ptr(),
        seqs.pos0.data_ptr(), seqs.slot.data_ptr(), q.data_ptr(), k.data_ptr(), v.data_ptr(), lg.data_ptr(),
        beta.data_ptr(), qk.data_ptr(), o.data_ptr(), state.S.data_ptr(), state.conv.data_ptr())
    dims = (ctypes.c_long * 15)(z.stride(0), a2.stride(0), *offs, sh.taps, G, H, K, V, sh.kp, B, T,
                                int(z.dtype == torch.float32))
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
