"""Projections ``x @ w.T`` of models whose sizes are not tuned one by one.

:class:`Projection` picks the kernel by the number of rows, as
:class:`kgs.serve.model.ServingModel` does for its tuned shapes: the skinny GEMM
over a prepacked weight for small decode batches, split-K four-wave tiles for
larger ones, the 256x256 pipeline for prompts, the library GEMM for shapes the
kernels do not take. A gated projection (fused gate|up weight) applies
``act(gate) * up`` (``act``: a name or a :class:`kgs.ops.activation.Gate`) in the
epilogue where one exists. fp32 runs on the library's
true fp32 GEMM.
"""
from __future__ import annotations

import torch

from . import decode as D
from .activation import Gate

SKINNY_MAX_ROWS = 32   # untuned shapes: skinny GEMM up to here
SPLIT_MAX_ROWS = 512   # four-wave split-K tiles up to here
TARGET_TILES = 400     # workgroups that fill the CUs about one and a half times
MAX_PARTIALS = 16 << 20  # fp32 partial products of a split-K call


def split_tiles(m: int, n: int, k: int) -> tuple[int, int, int] | None:
    """(tile width, K slices, tile height) of the four-wave GEMM for ``m`` rows, or
    None when the shape does not tile."""
    if n % 128 or k % 128:
        return None
    bm = 128 if m <= 128 else 256
    tiles = n // 128 * -(-m // bm)
    ns = 1
    while ns < 8 and 2 * ns * tiles <= TARGET_TILES and k % (256 * ns) == 0 and 2 * ns * m * n <= MAX_PARTIALS:
        ns *= 2
    return 128, ns, bm


class Projection:
    """``x @ w.T``, or ``act(x @ gate.T) * (x @ up.T)`` for ``gated=act`` with
    ``w = [gate; up]``. ``pack``: keep a second copy of the weight in the skinny
    GEMM's order for decode."""

    def __init__(self, w: torch.Tensor, gated=None, pack: bool = True):
        self.w, self.gated = w.contiguous(), None if gated is None else Gate.of(gated)
        if gated is not None and w.is_cuda:
            self.gated.limit_ptr(w.device)  # on the device before any hipGraph capture
        n, k = w.shape
        # every default skinny tile: 64 or 128 rows of w, 8 or 16 k-steps of 32
        fits = n % 128 == 0 and k % 512 == 0
        self.packed = None
        if pack and fits and w.dtype == torch.bfloat16 and w.is_cuda:
            self.packed = D.PackedWeight(self.w, swiglu=gated is not None, act=gated or "silu")

    def __call__(self, x: torch.Tensor) -> torch.Tensor:
        w, act = self.w, self.gated
        if x.dtype != w.dtype or x.shape[1] != w.shape[1]:
            raise ValueError(f"x {tuple(x.shape)} {x.dtype} does not fit w {tuple(w.shape)} {w.dtype}")
        m, (n, k) = x.shape[0], w.shape
        if x.dtype == torch.bfloat16:
            if m <= SKINNY_MAX_ROWS and self.packed is not None:
                return D.skinny_gemm(x, self.packed)
            if act is not None:
                y = self._gated(x, m)
                if y is not None:
                    return y
            else:
                y = self._plain(x, m, n, k)
                if y is not None:
                    return y
        elif torch.backends.cuda.matmul.allow_tf32:
            raise RuntimeError("fp32 projections need torch.backends.cuda.matmul.allow_tf32 = False")
        y = torch.matmul(x, w.T)
        if act is None:
            return y
        from .activation import act_mul

        return act_mul(y, act)

    def _gated(self, x, m):
        from .gemm import gemm_nt_w4x_swiglu, gemm_swiglu, swiglu_fused_ok

        if m > SPLIT_MAX_ROWS:
            return gemm_swiglu(x, self.w, self.gated)
        if not swiglu_fused_ok(x, self.w):
            return None
        return gemm_nt_w4x_swiglu(x, self.w, bn=128, bm=128 if m <= 128 else 256, nt_weights=D.NT_WEIGHTS,
                                  act=self.gated)

    def _plain(self, x, m, n, k):
        from .gemm import gemm_nt, gemm_nt_w4x

        if m > SPLIT_MAX_ROWS:
            return gemm_nt(x, self.w)
        if m < D.W4X_MIN_BATCH or x.stride(0) % 8 or x.data_ptr() % 16:
            return None
        route = D.w4x_route(m, n, k) or split_tiles(m, n, k)
        if route is None:
            return gemm_nt(x, self.w) if m >= 128 else None
        return gemm_nt_w4x(x, self.w, bn=route[0], nslice=route[1], bm=route[2], stages=D.w4x_stages(route),
                           nt_weights=D.w4x_nt(route))
