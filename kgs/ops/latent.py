"""Latent attention (``native/kernels/latent.hip``): every head's keys and values
are linear maps of one cached vector per token.

* :class:`LatentCache` -- pages ``[page][32 tokens][RP]`` per layer that has a
  latent of its own (layers that share one read its pages); where keys have a further
  part that turns with the position, one for all heads, it follows the latent in each
  row;
* :func:`latent_norm` -- both latents' RMS norms from the fused input projection,
  the cached one written to its slot, the rotated key part turned beside it;
* :func:`head_proj` -- the per-head products around the attention;
* :func:`latent_attention` -- the attention itself over the pages, in latent space:
  decoded tokens and short prompt portions (bf16: MFMA, split over the context;
  fp32 and latents above 512: the plain kernel), over the whole context or a window.

Long portions are cheaper on expanded keys and values:
:func:`kgs.ops.transformer.attention_ragged`.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _lib
from .decode import CUS, PAGE
from .hyper import _act, _f32

KERNEL_SIZES = (32, 64, 96, 128, 192, 256, 384, 512)  # latent sizes of the MFMA kernel
KERNEL_ROTS = (0, 32, 64)                             # and sizes of the rotated part
MAX_LATENT = 2048
MAX_ROT = 512
MAX_WAVES = 8


def padded_latent(n: int) -> int:
    """Columns of a cache row for a latent of size ``n``."""
    if n > MAX_LATENT:
        raise ValueError(f"latent size {n} is above {MAX_LATENT}")
    return next((s for s in KERNEL_SIZES if s >= n), (n + 31) // 32 * 32)


def padded_rot(n: int) -> int:
    """Columns of a cache row for a rotated key part of size ``n``."""
    if n > MAX_ROT:
        raise ValueError(f"rotated size {n} is above {MAX_ROT}")
    return (n + 31) // 32 * 32


def window_pages(window: int, queries: int = 1) -> int:
    """Most pages that ``queries`` consecutive query tokens with a window see together."""
    return (window + queries - 3) // PAGE + 2


class LatentCache:
    def __init__(self, sizes: dict[int, int], num_pages: int, dtype, device):
        """``sizes``: layer -> columns of a row (padded latent and rotated part)."""
        self.num_pages = num_pages
        # zeros: masked keys of a partly written page must be finite
        self.pages = {i: torch.zeros((num_pages, PAGE, rp), dtype=dtype, device=device) for i, rp in sizes.items()}

    @staticmethod
    def bytes_per_page(sizes: dict[int, int], itemsize: int) -> int:
        return PAGE * itemsize * sum(sizes.values())


@dataclass
class LatentRows:
    """The query tokens of one latent-attention call, numbered 0 .. nt-1, and the
    launch's shape. ``q0 / n / pos0 / bt`` per sequence (int32, device): its first
    token's number, tokens, first position, pages. ``rows``: the batch row of each
    token, None when they are the same. ``items``: (sequence, tile) pairs, None when
    every sequence has ``tiles`` tiles."""
    nt: int
    q0: torch.Tensor
    n: torch.Tensor
    pos0: torch.Tensor
    bt: torch.Tensor
    tok_seq: torch.Tensor
    tok_pos: torch.Tensor
    rows: torch.Tensor | None
    items: torch.Tensor | None
    ntiles: int
    tiles: int
    waves: int
    nsplit: int


def mfma_sizes(rp: int, hr: int) -> bool:
    """Whether the MFMA kernel takes a cache row (in bf16)."""
    return rp in KERNEL_SIZES and hr in KERNEL_ROTS


def split_count(ntiles: int, max_pages: int, rp: int = 0) -> int:
    """Context splits: as many workgroups as the CUs hold at once (two each, one
    where the page ring takes most of the LDS), at least two pages each."""
    return max(1, min((1 if rp > 384 else 2) * CUS // max(1, ntiles), (max_pages + 1) // 2, 64))


def waves_for(rows: int, rp: int) -> int:
    """Waves (of 16 rows) per workgroup for sequences of ``rows`` (token, head) rows."""
    return max(1, min(MAX_WAVES if rp <= 256 else MAX_WAVES // 2, (rows + 15) // 16))


def _turns(rotary, pos: torch.Tensor, n: int) -> tuple:
    """What the kernels need to turn by the int32 positions ``pos`` of ``n`` tokens
    (``rotary``: :class:`kgs.ops.talking.Rotary`): table, positions and sizes."""
    if pos.dtype != torch.int32 or not pos.is_contiguous() or not pos.is_cuda or pos.shape[0] < n:
        raise ValueError("rotary positions need contiguous int32 positions of the tokens")
    return rotary.table.data_ptr(), pos.data_ptr(), *rotary.table.shape


def latent_norm(z: torch.Tensor, oq: int, wq: torch.Tensor, qp: int, oc: int, wc: torch.Tensor | None,
                pages: torch.Tensor | None, slots: torch.Tensor, eps: float, rp: int = 0, okr: int = 0, rotary=None,
                pos: torch.Tensor | None = None) -> torch.Tensor:
    """RMS norms of the latents in ``z`` (query latent from column ``oq``, cached
    one from ``oc``): returns the query latent ``[T, qp]``, writes the other into
    ``pages`` at ``slots`` (-1: dropped). ``wc`` None: no latent of its own. ``rotary``: the
    columns from ``okr`` on, turned by the rows' ``pos``, follow the latent's ``rp``."""
    T = z.shape[0]
    hr = pages.shape[2] - rp if rotary is not None and wc is not None else 0
    nq, nc = wq.shape[0], 0 if wc is None else wc.shape[0]
    _act(z, T, max(oq + nq, oc + nc if nc else 0, okr + hr), z.dtype, "z")
    cq = torch.empty((T, qp), dtype=z.dtype, device=z.device)
    if nc and (pages.dtype != z.dtype or not pages.is_contiguous()):
        raise ValueError("pages must be contiguous and of z's dtype")
    turn = _turns(rotary, pos, T) if hr else (0, 0, 0, 0)
    rc = _lib.lib().kgs_latent_norm(z.data_ptr(), z.stride(0), oq, nq, qp, oc, nc, pages.shape[2] - hr if nc else 0,
                                    okr, hr, *turn, _f32(wq, (nq,), "wq"), _f32(wc, (nc,), "wc") if nc else 0,
                                    cq.data_ptr(), pages.data_ptr() if nc else 0, slots.data_ptr(), T, float(eps),
                                    int(z.dtype == torch.float32), _lib.stream_handle(z.device))
    _lib.check(rc, f"latent_norm[{T}]")
    return cq


def head_proj(a: torch.Tensor, w: torch.Tensor, nt: int, out: torch.Tensor, rows_in: torch.Tensor | None = None,
              rows_out: torch.Tensor | None = None, gate: torch.Tensor | None = None, each: bool = False,
              hr: int = 0, rotary=None, pos: torch.Tensor | None = None) -> torch.Tensor:
    """``out[rows_out[i], h] = (w[h] @ a[rows_in[i], h]) * sigmoid(gate[rows_out[i], h])``
    for ``a [R, H * K]``, ``w [H, N, K]``, ``out [R', >= H * N]``, i < nt. ``gate``: a column
    per head, or with ``each`` per output, ``H * N``. ``hr`` further columns of every head of ``a``, after
    its ``K``, go after the ``N`` of ``out``, turned by ``pos[i]`` (``rotary``)."""
    H, N, K = w.shape
    if a.dtype != w.dtype or out.dtype != w.dtype or not w.is_contiguous():
        raise ValueError("a, w and out must share a dtype, w contiguous")
    _act(a, a.shape[0], H * (K + hr), w.dtype, "a")
    _act(out, out.shape[0], H * (N + hr), w.dtype, "out")
    if (rows_in is None and a.shape[0] < nt) or (rows_out is None and out.shape[0] < nt):
        raise ValueError("fewer rows than tokens")
    rc = _lib.lib().kgs_head_proj(a.data_ptr(), w.data_ptr(), out.data_ptr(),
                                  0 if rows_in is None else rows_in.data_ptr(),
                                  0 if rows_out is None else rows_out.data_ptr(),
                                  0 if gate is None else _act(gate, gate.shape[0], H * N if each else H, w.dtype, "gate"),
                                  a.stride(0), K + hr, out.stride(0), N + hr, 0 if gate is None else gate.stride(0),
                                  N if each else 1, int(each),
                                  nt, H, N, K, hr, *(_turns(rotary, pos, nt) if hr else (0, 0, 0, 0)),
                                  int(w.dtype == torch.float32), _lib.stream_handle(a.device))
    _lib.check(rc, f"head_proj[{nt}x{H}x{N}x{K}]")
    return out


def latent_attention(q: torch.Tensor, pages: torch.Tensor, r: LatentRows, heads: int, scale: float, hr: int = 0,
                     window: int = 0) -> torch.Tensor:
    """Softmax attention of ``q [nt, H * (RP + hr)]`` (latent-space queries, each followed by
    its rotated part) over the cached rows up to each token's position -> ``[nt, H * RP]``.
    ``window``: a token sees itself and the ``window - 1`` before it (0: all)."""
    rp = pages.shape[2] - hr
    if q.dtype != pages.dtype or tuple(q.shape) != (r.nt, heads * (rp + hr)) or not q.is_contiguous() or \
            not pages.is_contiguous():
        raise ValueError(f"q {tuple(q.shape)} {q.dtype} does not fit {r.nt} x {heads} x {rp} + {hr} {pages.dtype}")
    o = torch.empty((r.nt, heads * rp), dtype=q.dtype, device=q.device)
    L, s = _lib.lib(), _lib.stream_handle(q.device)
    W = r.bt.shape[1]
    if q.dtype == torch.float32 or not mfma_sizes(rp, hr):
        rc = L.kgs_latent_attn_simple(q.data_ptr(), pages.data_ptr(), o.data_ptr(), r.tok_seq.data_ptr(),
                                      r.tok_pos.data_ptr(), r.bt.data_ptr(), heads, W, r.nt, rp, hr, window,
                                      float(scale), int(q.dtype == torch.float32), s)
        _lib.check(rc, f"latent_attention (plain) [{r.nt}x{heads}x{rp}]")
        return o
    po = ml = None
    if r.nsplit > 1:
        po = torch.empty((r.nsplit, r.nt * heads, rp), dtype=torch.float32, device=q.device)
        ml = torch.empty((r.nsplit, r.nt * heads, 2), dtype=torch.float32, device=q.device)
    rc = L.kgs_latent_attn(q.data_ptr(), pages.data_ptr(), o.data_ptr(), 0 if po is None else po.data_ptr(),
                           0 if ml is None else ml.data_ptr(), r.q0.data_ptr(), r.n.data_ptr(), r.pos0.data_ptr(),
                           r.bt.data_ptr(), 0 if r.items is None else r.items.data_ptr(), r.ntiles, r.tiles, r.waves,
                           r.nsplit, heads, W, r.nt, rp, hr, window, float(scale), s)
    _lib.check(rc, f"latent_attention[{r.nt}x{heads}x{rp}/{r.nsplit}]")
    return o
