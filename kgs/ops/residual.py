"""The fp32 residual between sublayers (``native/kernels/residual.hip``): what one
adds, and the next one's normed input, in one launch. fp32 and bf16 activations; the
residual is always fp32 ``[T, wp]``, padded with zero columns to a multiple of 8."""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _lib
from .hyper import _act, _f32

MAX_WIDTH = 16384


@dataclass(frozen=True)
class Norm:
    """RMS norm of ``groups`` equal consecutive parts, each by its own mean, times
    ``offset + w`` (1: weights stored around zero)."""
    width: int
    eps: float
    groups: int = 1
    offset: float = 1.0


@dataclass
class ExpertRows:
    """Outputs of a mixture of experts as :func:`residual_add` takes them: rows ``y``
    (``[P, wp]``, or fp32 partial products ``[slices, P, wp]``) and, per token and
    choice, its row (``pos [T, top]``, -1: none)."""
    y: torch.Tensor
    pos: torch.Tensor


@dataclass
class Scaled:
    """Rows ``[T, wp]`` of the activations' dtype, each times its number (fp32 ``[T]``)."""
    rows: torch.Tensor
    scale: torch.Tensor


@dataclass
class Embedding:
    """``scale * table[token]``, to be added to the residual."""
    tokens: torch.Tensor
    table: torch.Tensor
    scale: float


MAX_SCALED = 2


def _tokens(t: torch.Tensor, T: int) -> int:
    if t.dtype != torch.int32 or not t.is_contiguous() or not t.is_cuda or t.shape[0] != T:
        raise ValueError("tokens must be contiguous int32 on the GPU")
    return t.data_ptr()


def _zero(t: torch.Tensor | None) -> tuple[int, int]:
    if t is None:
        return 0, 0
    if t.dtype != torch.int32 or not t.is_contiguous() or not t.is_cuda:
        raise ValueError("counters to clear must be contiguous int32 on the GPU")
    return t.data_ptr(), t.numel()


def residual_embed(tokens: torch.Tensor, embed: torch.Tensor, scale: float, w: torch.Tensor, norm: Norm,
                   zero: torch.Tensor | None = None) -> tuple[torch.Tensor, torch.Tensor]:
    """Start the residual: ``x = scale * embed[token]``. Returns (x fp32 ``[T, wp]``,
    the first layer's normed input in the table's dtype); ``zero``: counters cleared."""
    T, wp = tokens.shape[0], w.shape[0]
    x = torch.empty((T, wp), dtype=torch.float32, device=tokens.device)
    h = torch.empty((T, wp), dtype=embed.dtype, device=tokens.device)
    rc = _lib.lib().kgs_residual_embed(x.data_ptr(), _tokens(tokens, T), _act(embed, embed.shape[0], wp, h.dtype, "embed"),
                                       embed.stride(0), float(scale), _f32(w, (wp,), "w"), h.data_ptr(), h.stride(0),
                                       *_zero(zero), T, norm.width, wp, norm.groups, float(norm.offset), float(norm.eps),
                                       int(h.dtype == torch.float32), _lib.stream_handle(x.device))
    _lib.check(rc, f"residual_embed[{T}x{wp}]")
    return x, h


def residual_add(x: torch.Tensor, a: torch.Tensor | None, bias: torch.Tensor | None, experts: ExpertRows | None,
                 w: torch.Tensor, norm: Norm, dtype, zero: torch.Tensor | None = None, scaled=(),
                 embedding: Embedding | None = None) -> torch.Tensor:
    """``x += a + bias + every token's expert rows + scaled rows + embedding`` in place
    (``scaled``: up to two :class:`Scaled`), then the normed input of what comes next."""
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
    if len(scaled) > MAX_SCALED:
        raise ValueError(f"{len(scaled)} scaled inputs are above {MAX_SCALED}")
    more = []
    for i in range(MAX_SCALED):
        s = scaled[i] if i < len(scaled) else None
        more += [0, 0, 0] if s is None else [_act(s.rows, T, wp, dtype, "rows"), s.rows.stride(0), _f32(s.scale, (T,), "scale")]
    e = embedding
    again = [0, 0, 0, 0.0] if e is None else [_tokens(e.tokens, T), _act(e.table, e.table.shape[0], wp, dtype, "embed"),
                                              e.table.stride(0), float(e.scale)]
    rc = _lib.lib().kgs_residual_add(_f32(x, (T, wp), "x"), 0 if a is None else _act(a, T, wp, dtype, "a"),
                                     0 if a is None else a.stride(0), 0 if bias is None else _f32(bias, (wp,), "bias"),
                                     y, ldy, ys, ns, y32, pos, top, *more, *again, _f32(w, (wp,), "w"), h.data_ptr(),
                                     h.stride(0), *_zero(zero), T, norm.width, wp, norm.groups, float(norm.offset),
                                     float(norm.eps), int(f32), _lib.stream_handle(x.device))
    _lib.check(rc, f"residual_add[{T}x{wp}]")
    return h
