"""Hyper-connections (``native/kernels/hyper.hip``): the fp32 residual streams'
write-back, read-out and pre-norm between two sublayers as one launch. fp32 and
bf16 activations; the streams are always fp32 ``[T, S, D]``."""
from __future__ import annotations

import torch

from . import _lib

MAX_STREAMS = 8


def _f32(t: torch.Tensor, shape: tuple, name: str) -> int:
    if t.dtype != torch.float32 or tuple(t.shape) != shape or not t.is_contiguous() or not t.is_cuda:
        raise ValueError(f"{name} must be a contiguous fp32 GPU tensor of shape {shape}, got {t.dtype} {tuple(t.shape)}")
    return t.data_ptr()


def _act(t: torch.Tensor, rows: int, cols: int, dtype, name: str) -> int:
    if t.dtype != dtype or t.dim() != 2 or t.shape[0] != rows or t.shape[1] < cols or t.stride(1) != 1 or not t.is_cuda:
        raise ValueError(f"{name} must be a row-major {dtype} GPU matrix [{rows}, >= {cols}], got {t.dtype} "
                         f"{tuple(t.shape)}")
    return t.data_ptr()


def _out(out, rows: int, ld: int, dtype, device) -> torch.Tensor:
    if dtype not in (torch.bfloat16, torch.float32):
        raise TypeError(f"activations must be bf16 or fp32, got {dtype}")
    return torch.empty((rows, ld), dtype=dtype, device=device) if out is None else out


def hyper_embed(tokens: torch.Tensor, embed: torch.Tensor, w0: torch.Tensor, w_in: torch.Tensor, w: torch.Tensor,
                width: int, eps: float, ld: int | None = None) -> tuple[torch.Tensor, torch.Tensor]:
    """Start the streams: all equal to ``rmsnorm(embed[token]) * w0``. Returns
    (streams ``[T, S, D]`` fp32, the first sublayer's input ``[T, ld]`` in the
    table's dtype, zero past ``width``)."""
    T, S = tokens.shape[0], w_in.shape[0]
    if tokens.dtype != torch.int32 or not tokens.is_contiguous() or not tokens.is_cuda:
        raise ValueError("tokens must be contiguous int32 on the GPU")
    x = torch.empty((T, S, width), dtype=torch.float32, device=tokens.device)
    h = _out(None, T, ld or width, embed.dtype, tokens.device)
    _act(embed, embed.shape[0], width, h.dtype, "embed")
    rc = _lib.lib().kgs_hyper_embed(x.data_ptr(), tokens.data_ptr(), embed.data_ptr(), _f32(w0, (width,), "w0"),
                                    _f32(w_in, (S,), "w_in"), _f32(w, (width,), "w"), h.data_ptr(), T, S, width,
                                    embed.stride(0), h.stride(0), float(eps), int(h.dtype == torch.float32),
                                    _lib.stream_handle(x.device))
    _lib.check(rc, f"hyper_embed[{T}x{S}x{width}]")
    return x, h


def hyper_step(x: torch.Tensor, y: torch.Tensor | None, mix: torch.Tensor | None, w_out: torch.Tensor | None,
               w_in: torch.Tensor, w: torch.Tensor, eps: float, dtype=None, ld: int | None = None) -> torch.Tensor:
    """``x_t <- sum_s mix[s, t] x_s + w_out[t] y`` in place (``y`` None: unchanged),
    then ``rmsnorm(sum_s w_in[s] x_s) * w`` as ``[T, ld]`` (zero past the width)."""
    T, S, D = x.shape
    _f32(x, (T, S, D), "x")
    dtype = dtype or (y.dtype if y is not None else torch.bfloat16)
    h = _out(None, T, ld or D, dtype, x.device)
    yp = 0 if y is None else _act(y, T, D, dtype, "y")
    rc = _lib.lib().kgs_hyper_step(x.data_ptr(), yp, 0 if y is None else _f32(mix, (S, S), "mix"),
                                   0 if y is None else _f32(w_out, (S,), "w_out"), _f32(w_in, (S,), "w_in"),
                                   _f32(w, (D,), "w"), h.data_ptr(), T, S, D, 0 if y is None else y.stride(0),
                                   h.stride(0), float(eps), int(dtype == torch.float32), _lib.stream_handle(x.device))
    _lib.check(rc, f"hyper_step[{T}x{S}x{D}]")
    return h
