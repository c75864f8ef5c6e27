"""Projections ``x @ w.T`` of models whose sizes are not tuned one by one: bf16 on
the MFMA GEMMs of :mod:`kgs.ops.gemm` for prompt-sized batches and on the
library GEMM for decode-sized ones (the split of
:class:`kgs.serve.model.ServingModel`), fp32 on the library's true fp32 GEMM."""
from __future__ import annotations

import torch

from . import decode as D

GEMM_MIN_ROWS = 128  # from here on the 256x256 pipeline


def project(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    if x.dtype != w.dtype or x.shape[1] != w.shape[1]:
        raise ValueError(f"x {tuple(x.shape)} {x.dtype} does not fit w {tuple(w.shape)} {w.dtype}")
    m, (n, k) = x.shape[0], w.shape
    if x.dtype == torch.float32:
        if torch.backends.cuda.matmul.allow_tf32:
            raise RuntimeError("fp32 projections need torch.backends.cuda.matmul.allow_tf32 = False")
        return torch.matmul(x, w.T)
    if m >= GEMM_MIN_ROWS:
        from .gemm import gemm_nt

        return gemm_nt(x, w)
    route = D.w4x_route(m, n, k)
    if route is not None:
        from .gemm import gemm_nt_w4x

        return gemm_nt_w4x(x, w, bn=route[0], nslice=route[1], bm=route[2], stages=D.w4x_stages(route),
                           nt_weights=D.w4x_nt(route))
    return torch.matmul(x, w.T)
