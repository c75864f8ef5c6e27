"""Softmax attention over head pages (``native/kernels/paged.hip``): the paged cache of
:mod:`kgs.ops.talking`, grouped key heads, causal, optionally chunked (a query sees the
keys of its own chunk of positions only, and reads only their pages).

Differential heads (:class:`Differential`) hold two queries and two keys each, whose softmaxes
weigh the same values.

* :func:`paged_heads` -- the sizes of a layer; pages, projections' biases and rotary
  positions are :class:`kgs.ops.talking.HeadPages` and :func:`kgs.ops.talking.write_kv`;
* :func:`paged_rows` -- single query tokens (decode, short portions), split over the
  visible pages; :func:`paged_tiles` -- prompt portions.
"""
from __future__ import annotations

from dataclasses import dataclass

import numpy as np
import torch

from . import _lib
from .decode import CUS, PAGE
from .hyper import _act
from .talking import MFMA_DIMS, Heads, QueryRows, padded_dim

TILE_ROWS = 128       # (query, head of the group) rows of a tile
MAX_PLAIN_VDIM = 1024


@dataclass(frozen=True)
class Differential:
    """How the two maps of differential heads are joined: ``o = a1 - lam a2``, then ``post o /
    sqrt(mean o^2 + eps)`` over a head's ``vdim`` values."""
    lam: float
    post: float
    vdim: int
    eps: float


def _joined(h: Heads, d: Differential | None) -> tuple:
    if (d is not None) != (h.maps == 2):
        raise ValueError(f"heads of {h.maps} maps")
    return (h.maps, h.dvp, 0.0, 0.0, 0.0) if d is None else (h.maps, d.vdim, float(d.lam), float(d.post), float(d.eps))


def paged_heads(heads: int, kv_heads: int, dim: int, vdim: int, dtype, maps: int = 1) -> Heads:
    """``dim``: query / key size (of one map)."""
    dkp, dvp = padded_dim(dim), padded_dim(vdim)
    mfma = dtype == torch.bfloat16 and dkp in MFMA_DIMS and dvp in MFMA_DIMS
    if not mfma and dvp > MAX_PLAIN_VDIM:
        raise ValueError(f"value size {vdim} is above {MAX_PLAIN_VDIM}")
    return Heads(heads, kv_heads, maps * dkp, dvp, mfma, maps)


def tile_queries(h: Heads) -> int:
    """Queries of a tile; 0: no tiled kernel for these heads."""
    return TILE_ROWS // h.maps // h.group if h.mfma else 0


@dataclass
class Portions:
    """Blocks of up to :func:`tile_queries` consecutive queries: int32 ``[n, 4]`` (first
    batch row, block-table row, position of the first, queries)."""
    items: torch.Tensor
    bt: torch.Tensor


def portion_items(portions, tile: int, chunk: int) -> np.ndarray:
    """Items of ``portions`` (first batch row, block-table row, position, tokens), the
    ones with the most keys first."""
    b = np.array([(r + j, s, p + j, min(tile, n - j)) for r, s, p, n in portions for j in range(0, n, tile)], np.int64)
    first = b[:, 2] - b[:, 2] % chunk if chunk else 0
    return b[np.argsort(first - b[:, 2] - b[:, 3], kind="stable")]


def row_splits(n: int, kv_heads: int, group: int, pages: int, maps: int = 1) -> int:
    """Splits of the visible pages: two workgroups of four waves per CU (what fits), at least two
    pages per wave."""
    units = n * kv_heads * -(-group * maps // 16)
    return max(1, min(2 * CUS // max(1, units), -(-pages // 8), 64))


def visible_pages(pos: int, chunk: int) -> int:
    """Pages a query at ``pos`` reads."""
    return pos // PAGE + 1 - (pos - pos % chunk if chunk else 0) // PAGE


def paged_rows(q: torch.Tensor, pages: torch.Tensor, h: Heads, scale: float, chunk: int, r: QueryRows,
               out: torch.Tensor, diff: Differential | None = None) -> torch.Tensor:
    """Attention of single query tokens over their sequences' pages up to their positions;
    ``q [T, >= H dkp]``, ``out [T, >= H dvp]``; ``chunk`` 0: none; ``diff``: for heads of two maps."""
    po = pml = None
    ns = r.nsplit if h.mfma else 1
    if ns > 1:
        po = torch.empty((r.n, ns, h.heads * h.maps, h.dvp), dtype=torch.float32, device=q.device)
        pml = torch.empty((r.n, ns, h.heads * h.maps, 2), dtype=torch.float32, device=q.device)
    rc = _lib.lib().kgs_paged_rows(_act(q, q.shape[0], h.heads * h.dkp, pages.dtype, "q"), q.stride(0), pages.data_ptr(),
                                   _act(out, out.shape[0], h.heads * h.dvp, pages.dtype, "out"), out.stride(0),
                                   r.bt.data_ptr(), r.bt.shape[1], r.tok_seq.data_ptr(), r.tok_pos.data_ptr(),
                                   0 if r.rows is None else r.rows.data_ptr(), 0 if po is None else po.data_ptr(),
                                   0 if pml is None else pml.data_ptr(), float(scale), chunk, r.n, h.heads, h.kv_heads,
                                   h.dkp, h.dvp, *_joined(h, diff), ns, int(not h.mfma), int(q.dtype == torch.float32),
                                   _lib.stream_handle(q.device))
    _lib.check(rc, f"paged_rows[{r.n}x{h.heads}/{ns}]")
    return out


def paged_tiles(q: torch.Tensor, pages: torch.Tensor, h: Heads, scale: float, chunk: int, t: Portions,
                out: torch.Tensor, diff: Differential | None = None) -> torch.Tensor:
    """Attention of prompt portions (:class:`Portions`), as :func:`paged_rows`."""
    if not tile_queries(h):
        raise ValueError(f"{h} has no tiled kernel")
    if t.items.dtype != torch.int32 or t.items.dim() != 2 or t.items.shape[1] != 4 or not t.items.is_contiguous():
        raise ValueError("items must be contiguous int32 [n, 4]")
    rc = _lib.lib().kgs_paged_tiles(_act(q, q.shape[0], h.heads * h.dkp, torch.bfloat16, "q"), q.stride(0),
                                    pages.data_ptr(), _act(out, out.shape[0], h.heads * h.dvp, torch.bfloat16, "out"),
                                    out.stride(0), t.bt.data_ptr(), t.bt.shape[1], t.items.data_ptr(), t.items.shape[0],
                                    float(scale), chunk, h.heads, h.kv_heads, h.dkp, h.dvp, *_joined(h, diff),
                                    _lib.stream_handle(q.device))
    _lib.check(rc, f"paged_tiles[{t.items.shape[0]}x{h.heads}]")
    return out
