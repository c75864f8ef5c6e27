"""Elementwise steps around the projections (``native/kernels/activation.hip``),
bf16 or fp32: the gated feed-forward product, the normed powers of a feed-forward row and
the logits' soft cap."""
from __future__ import annotations

from dataclasses import dataclass
from functools import lru_cache

import torch

from . import _lib

ACTS = {"silu": 0, "gelu_tanh": 1, "clamped": 2}


@dataclass(frozen=True)
class Gate:
    """How a gated feed-forward joins its two projections: ``silu(gate) * up``,
    ``gelu_tanh(gate) * up``, or ``clamped``: ``g sigmoid(1.702 g) (u + 1)`` with
    ``g = min(gate, limit)``, ``u = clamp(up, -limit, limit)``."""
    act: str
    limit: float = 0.0

    def __post_init__(self):
        if self.act not in ACTS:
            raise ValueError(f"unknown gate activation {self.act!r}")

    @classmethod
    def of(cls, act) -> "Gate":
        return act if isinstance(act, Gate) else cls(act)

    def limit_ptr(self, device) -> int:
        """The limit on the device, for epilogues that read it there (0: none)."""
        return _limit(self.limit, str(device)).data_ptr() if self.act == "clamped" else 0


@lru_cache(maxsize=None)
def _limit(limit: float, device: str) -> torch.Tensor:
    return torch.tensor([limit], dtype=torch.float32, device=device)


def _mat(t: torch.Tensor, name: str) -> None:
    if t.dtype not in (torch.bfloat16, torch.float32) or t.dim() != 2 or t.stride(1) != 1 or not t.is_cuda:
        raise ValueError(f"{name} must be a row-major bf16 or fp32 GPU matrix")


def act_mul(gu: torch.Tensor, act) -> torch.Tensor:
    """``act(gu[:, :n]) * gu[:, n:]`` for a fused gate|up output of width 2n (``act``: a
    name or a :class:`Gate`)."""
    _mat(gu, "gu")
    gate = Gate.of(act)
    rows, n = gu.shape[0], gu.shape[1] // 2
    out = torch.empty((rows, n), dtype=gu.dtype, device=gu.device)
    rc = _lib.lib().kgs_act_mul(gu.data_ptr(), out.data_ptr(), rows, n, gu.stride(0), n, ACTS[gate.act], float(gate.limit),
                                int(gu.dtype == torch.float32), _lib.stream_handle(gu.device))
    _lib.check(rc, f"act_mul[{rows}x{n}]")
    return out


def poly_norm(z: torch.Tensor, c: torch.Tensor, n: int, eps: float) -> torch.Tensor:
    """``c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3`` row by row, N dividing by the root mean square
    of the row's first ``n`` values (the others are zero padding); ``c`` fp32 ``[4]``."""
    _mat(z, "z")
    if c.dtype != torch.float32 or tuple(c.shape) != (4,) or not c.is_cuda:
        raise ValueError("c must be four fp32 numbers on the GPU")
    rows, cols = z.shape
    out = torch.empty((rows, cols), dtype=z.dtype, device=z.device)
    rc = _lib.lib().kgs_poly_norm(z.data_ptr(), z.stride(0), c.data_ptr(), out.data_ptr(), cols, rows, n, cols, float(eps),
                                  int(z.dtype == torch.float32), _lib.stream_handle(z.device))
    _lib.check(rc, f"poly_norm[{rows}x{n}]")
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
