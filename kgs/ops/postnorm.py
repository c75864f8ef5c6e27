"""The fp32 residual of layers that norm what a sublayer puts out and convolve what a mixer
reads over time (``native/kernels/postnorm.hip``): a sublayer's normed output is added, and
the next one's input made, in one launch. fp32 and bf16 activations; the residual is
always fp32 ``[T, wp]``, padded with zero columns to a multiple of 8.

* :class:`ConvState` -- per slot the last inputs of one layer's convolution;
* :class:`Conv` -- its weights, as the kernel reads them;
* :class:`PostNorm` -- the residual of one step through all sublayers.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _lib
from .delta import RaggedSeqs
from .hyper import _act, _f32
from .residual import _tokens

MAX_WIDTH = 16384


class ConvState:
    """fp32 ``[slots, taps - 1, wp]``: the input at position p in entry ``p % (taps - 1)``. A
    portion at position 0 ignores what its slot holds."""

    def __init__(self, taps: int, wp: int, slots: int, device):
        self.rows = torch.zeros((slots, max(1, taps - 1), wp), dtype=torch.float32, device=device)

    @staticmethod
    def bytes_per_slot(taps: int, wp: int) -> int:
        return 4 * max(1, taps - 1) * wp


class Conv:
    """``w [width, taps]``, the last tap on the row itself."""

    def __init__(self, w: torch.Tensor, wp: int):
        self.taps = w.shape[1]
        w = torch.nn.functional.pad(w.float().flip(1).T, (0, wp - w.shape[0]))
        self.w = w.contiguous()  # [taps, wp]: row d the weight of the row d before


@dataclass
class Sublayer:
    """What a sublayer put out and the number its norm is scaled by."""
    y: torch.Tensor
    gain: float


class PostNorm:
    """The residual of one batch. ``add(sublayer, conv, state)`` adds a sublayer's normed output
    and returns the next mixer's input; without ``conv`` the next feed-forward's;
    :meth:`close` adds the last one and returns the normed input of the output projection.
    ``save``: the state that keeps the inputs the added sublayer's mixer has read."""

    def __init__(self, tokens: torch.Tensor, seqs: RaggedSeqs, width: int, wp: int, eps: float, dtype):
        self.tokens, self.seqs, self.width, self.wp, self.eps, self.dtype = tokens, seqs, width, wp, eps, dtype
        self.x = self._spare = None

    def _new(self, dtype):
        return torch.empty((self.tokens.shape[0], self.wp), dtype=dtype, device=self.tokens.device)

    def _step(self, table, sub, conv, state, final, save):
        T, seqs, f32 = self.tokens.shape[0], self.seqs, self.dtype == torch.float32
        h = self._new(self.dtype)
        moves = conv is not None and conv.taps > 1
        if self.x is None:
            self.x = self._new(torch.float32)
            src, dst = None, self.x
        elif moves:  # rows of x are read by more than one workgroup
            src, dst = self.x, self._new(torch.float32) if self._spare is None else self._spare
            self._spare, self.x = self.x, dst
        else:
            src = dst = self.x
        first = [0, 0, 0] if table is None else [_tokens(self.tokens, T), _act(table, table.shape[0], self.wp, self.dtype, "embed"),
                                                 table.stride(0)]
        added = [0, 0, 0.0] if sub is None else [_act(sub.y, T, self.wp, self.dtype, "y"), sub.y.stride(0), float(sub.gain)]
        taps = conv.taps if conv is not None else save.rows.shape[1] + 1 if save is not None else 1
        for s in (state, save):
            if s is not None and (s.rows.shape[1:] != (max(1, taps - 1), self.wp) or not s.rows.is_contiguous()):
                raise ValueError(f"state {tuple(s.rows.shape)} does not fit {taps} taps")
        rc = _lib.lib().kgs_postnorm(
            0 if src is None else _f32(src, (T, self.wp), "x"), dst.data_ptr(), *first, *added, float(self.eps),
            0 if conv is None else _f32(conv.w, (taps, self.wp), "conv"), state.rows.data_ptr() if moves else 0, taps,
            int(final is not None), float(final or 0.0), 0 if save is None else save.rows.data_ptr(),
            seqs.row_seq.data_ptr(), seqs.row0.data_ptr(), seqs.n.data_ptr(), seqs.pos0.data_ptr(), seqs.slot.data_ptr(),
            h.data_ptr(), h.stride(0), T, self.width, self.wp, int(f32),
            _lib.stream_handle(h.device))
        _lib.check(rc, f"postnorm[{T}x{self.wp}]")
        return h

    def start(self, table: torch.Tensor, conv: Conv, state: ConvState | None) -> torch.Tensor:
        """``x = table[token]``; returns the first mixer's input."""
        return self._step(table, None, conv, state, None, None)

    def add(self, sub: Sublayer, conv: Conv | None = None, state: ConvState | None = None,
            save: ConvState | None = None) -> torch.Tensor:
        return self._step(None, sub, conv, state, None, save)

    def close(self, sub: Sublayer, gain: float, save: ConvState | None = None) -> torch.Tensor:
        return self._step(None, sub, None, None, gain, save)
