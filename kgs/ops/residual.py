"""The fp32 residual between layers (``native/kernels/residual.hip``): what a layer
adds, and the next layer's normed input, in one launch. The norm's weight is stored
around zero. fp32 and bf16 activations; the residual is always fp32 ``[T, wp]``,
padded with zero columns to a multiple of 8."""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _lib
from .hyper import _act, _f32

MAX_WIDTH = 16384


@dataclass
class ExpertRows:
    """Outputs of a mixture of experts as :func:`residual_add` takes them: rows ``y``
    (``[P, wp]``, or fp32 partial products ``[slices, P, wp]``) and, per token and
    choice, its row (``pos [T, top]``, -1: none)."""
    y: torch.Tensor
    pos: torch.Tensor


def _zero(t: torch.Tensor | None) -> tuple[int, int]:
    if t is None:
        return 0, 0
    if t.dtype != torch.int32 or not t.is_contiguous() or not t.is_cuda:
        raise ValueError("counters to clear must be contiguous int32 on the GPU")
    return t.data_ptr(), t.numel()


def residual_embed(tokens: torch.Tensor, embed: torch.Tensor, scale: float, w: torch.Tensor, width: int, eps: float,
                   zero: torch.Tensor | None = None) -> tuple[torch.Tensor, torch.Tensor]:
    """Start the residual: ``x = scale * embed[token]``. Returns (x fp32 ``[T, wp]``,
    the first layer's normed input in the table's dtype); ``zero``: counters cleared."""
    T, wp = tokens.shape[0], w.shape[0]
    if tokens.dtype != torch.int32 or not tokens.is_contiguous() or not tokens.is_cuda:
        raise ValueError("tokens must be contiguous int32 on the GPU")
    x = torch.empty((T, wp), dtype=torch.float32, device=tokens.device)
    h = torch.empty((T, wp), dtype=embed.dtype, device=tokens.device)
    rc = _lib.lib().kgs_residual_embed(x.data_ptr(), tokens.data_ptr(), _act(embed, embed.shape[0], wp, h.dtype, "embed"),
                                       embed.stride(0), float(scale), _f32(w, (wp,), "w"), h.data_ptr(), h.stride(0),
                                       *_zero(zero), T, width, wp, float(eps), int(h.dtype == torch.float32),
                                       _lib.stream_handle(x.device))
    _lib.check(rc, f"residual_embed[{T}x{wp}]")
    return x, h


def residual_add(x: torch.Tensor, a: torch.Tensor | None, bias: torch.Tensor | None, experts: ExpertRows | None,
                 w: torch.Tensor, width: int, eps: float, dtype, zero: torch.Tensor | None = None) -> torch.Tensor:
    """``x += a + bias + every token's expert rows`` in place, then the normed input of
    what comes next."""
    T, wp = x.shape
    f32 = dtype == torch.float32
    h = torch.empty((T, wp), dtype=dtype, device=x.device)
    y, ldy, ys, ns, y32, pos, top = 0, 0, 0, 0, 0, 0, 0
    if experts is not None:
        t = experts.y
        if t.dtype not in (dtype, torch.float32) or not t.is_contiguous() or t.shape[-1] != wp:
            raise ValueError(f"expert rows {tuple(t.shape)} {t.dtype} do not fit width {wp}")
        if experts.pos.dtype != torch.int32 or not experts.pos.is_contiguous() or experts.pos.shape[0] != T:
            raise ValueError("pos must be contiguous int32 [T, top]")
        y, ldy, y32 = t.data_ptr(), wp, int(t.dtype == torch.float32)
        ns, ys = (t.shape[0], t.shape[1] * wp) if t.dim() == 3 else (1, 0)
        pos, top = experts.pos.data_ptr(), experts.pos.shape[1]
    rc = _lib.lib().kgs_residual_add(_f32(x, (T, wp), "x"), 0 if a is None else _act(a, T, wp, dtype, "a"),
                                     0 if a is None else a.stride(0), 0 if bias is None else _f32(bias, (wp,), "bias"),
                                     y, ldy, ys, ns, y32, pos, top, _f32(w, (wp,), "w"), h.data_ptr(), h.stride(0),
                                     *_zero(zero), T, width, wp, float(eps), int(f32), _lib.stream_handle(x.device))
    _lib.check(rc, f"residual_add[{T}x{wp}]")
    return h
