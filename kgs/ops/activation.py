"""Elementwise steps around the projections (``native/kernels/activation.hip``),
bf16 or fp32: the gated feed-forward product and the logits' soft cap."""
from __future__ import annotations

import torch

from . import _lib

ACTS = {"silu": 0, "gelu_tanh": 1}


def _mat(t: torch.Tensor, name: str) -> None:
    if t.dtype not in (torch.bfloat16, torch.float32) or t.dim() != 2 or t.stride(1) != 1 or not t.is_cuda:
        raise ValueError(f"{name} must be a row-major bf16 or fp32 GPU matrix")


def act_mul(gu: torch.Tensor, act: str) -> torch.Tensor:
    """``act(gu[:, :n]) * gu[:, n:]`` for a fused gate|up output of width 2n."""
    _mat(gu, "gu")
    rows, n = gu.shape[0], gu.shape[1] // 2
    out = torch.empty((rows, n), dtype=gu.dtype, device=gu.device)
    rc = _lib.lib().kgs_act_mul(gu.data_ptr(), out.data_ptr(), rows, n, gu.stride(0), n, ACTS[act],
                                int(gu.dtype == torch.float32), _lib.stream_handle(gu.device))
    _lib.check(rc, f"act_mul[{rows}x{n}]")
    return out


def softcap(x: torch.Tensor, cols: int, cap: float) -> torch.Tensor:
    """fp32 ``cap * tanh(x[:, :cols] / cap)`` (``cap`` 0: only the conversion)."""
    _mat(x, "x")
    rows = x.shape[0]
    if x.shape[1] < cols:
        raise ValueError("x has fewer columns than asked for")
    out = torch.empty((rows, cols), dtype=torch.float32, device=x.device)
    for r in range(0, rows, 65535):
        n = min(65535, rows - r)
        rc = _lib.lib().kgs_softcap(x[r:].data_ptr(), out[r:].data_ptr(), n, cols, x.stride(0), float(cap),
                                    int(x.dtype == torch.float32), _lib.stream_handle(x.device))
        _lib.check(rc, f"softcap[{n}x{cols}]")
    return out
