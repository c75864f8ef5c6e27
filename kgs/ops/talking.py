"""Talking-heads attention over a paged grouped-head cache
(``native/kernels/talking.hip``): scores of all heads mixed by a learned matrix, a
learned bias per distance bucket, one added to the softmax's denominator.

* :class:`HeadPages` -- per layer ``[page][kv head][K 32 x dkp | V 32 x dvp]`` in MFMA
  fragment order;
* :class:`TalkingWeights` -- what the kernels need of the mixing matrix, the
  temperatures and the distance table;
* :func:`write_kv` -- the projections' biases and the cache write;
* :func:`attention_rows` -- single query tokens (decode, short portions), split over
  the context; :func:`attention_tiles` -- prompt portions, 16 or 32 queries per workgroup.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from fractions import Fraction

import numpy as np
import torch

from . import _lib
from .decode import CUS, PAGE
from .hyper import _act, _f32

LOG2E = 1.4426950408889634
MFMA_DIMS = (64, 128)   # head sizes of the MFMA kernels (others are padded up, larger ones run plain)
MAX_ROW_HEADS = 64      # heads of the MFMA rows kernel
MAX_SLOTS = 8           # slots of 4 heads of the tiles kernel


def padded_dim(n: int) -> int:
    return next((s for s in MFMA_DIMS if s >= n), (n + 31) // 32 * 32)


@dataclass(frozen=True)
class Heads:
    """Sizes of one attention layer. Query head h reads key head ``h // (heads // kv_heads)``."""
    heads: int
    kv_heads: int
    dkp: int             # padded query / key size
    dvp: int             # padded value size
    mfma: bool           # the MFMA kernels take it (bf16)
    maps: int = 1        # 2: differential heads, dkp holds the keys of both maps

    @property
    def group(self) -> int:
        return self.heads // self.kv_heads

    @property
    def slots(self) -> int:
        return self.kv_heads * -(-self.group // 4)

    @property
    def tiled(self) -> bool:
        return self.mfma and self.slots <= MAX_SLOTS

    @property
    def tile(self) -> int:
        """Queries of one tile (a workgroup, one per CU)."""
        return 32 if self.slots <= 4 else 16

    @property
    def tile_bytes(self) -> int:
        """Scratch of one tile: its queries in operand order."""
        form = 2 if self.slots <= 2 else 4 if self.slots <= 4 else 8
        return form * 256 * self.tile * (self.dkp // 32)

    def slot_heads(self) -> list[int]:
        """Head at every position of the slots (-1: empty), padded to whole 16s."""
        out = []
        for g in range(self.kv_heads):
            for c in range(-(-self.group // 4) * 4):
                out.append(g * self.group + c if c < self.group else -1)
        return out + [-1] * (-len(out) % 16)


def heads_of(heads: int, kv_heads: int, dim: int, vdim: int, dtype) -> Heads:
    dkp, dvp = padded_dim(dim), padded_dim(vdim)
    mfma = (dtype == torch.bfloat16 and heads <= MAX_ROW_HEADS and dkp in MFMA_DIMS and dvp in MFMA_DIMS)
    return Heads(heads, kv_heads, dkp, dvp, mfma)


class HeadPages:
    def __init__(self, layers: dict[int, Heads], num_pages: int, dtype, device):
        self.num_pages = num_pages
        # zeros: masked keys of a partly written page must be finite
        self.pages = {i: torch.zeros((num_pages, h.kv_heads, PAGE * (h.dkp + h.dvp)), dtype=dtype, device=device)
                      for i, h in layers.items()}

    @staticmethod
    def bytes_per_page(layers: dict[int, Heads], itemsize: int) -> int:
        return PAGE * itemsize * sum(h.kv_heads * (h.dkp + h.dvp) for h in layers.values())


def buckets(rows: int, far: float, n: int) -> np.ndarray:
    """Bucket of the distances 0 .. n-1: ``rows // 2`` single distances, then
    logarithmic ones up to ``far``, decided in exact arithmetic: bucket ``half + k``
    starts where ``(n / half) ** half >= (far / half) ** k``."""
    half, f = rows // 2, Fraction(far)
    out, k = np.zeros(n, np.int64), 0
    for i in range(n):
        if i < half:
            out[i] = i
            continue
        # (i / half)^half >= (far / half)^(k + 1)
        while half + k < rows - 1 and Fraction(i, half) ** half >= (f / half) ** (k + 1):
            k += 1
        out[i] = half + k
    return out


def mix_fragments(t: torch.Tensor, order: list[int]) -> torch.Tensor:
    """MFMA fragments of the mixing matrix ``t [H, H]`` for heads in ``order`` (a
    multiple of 16 positions, -1 empty): ``[out tiles][chunks of 32][64 lanes][8]``,
    lane 16 q + n = output n of the tile, element e = position 16 (e // 4) + 4q + e % 4."""
    P = len(order)
    chunks = -(-P // 32)
    pad = torch.zeros((P, chunks * 32), dtype=t.dtype, device=t.device)
    have = [i for i, h in enumerate(order) if h >= 0]
    idx = torch.tensor([order[i] for i in have], device=t.device)
    at = torch.tensor(have, device=t.device)
    pad[at[:, None], at[None]] = t[idx][:, idx]
    # [tile, n, chunk, hi, q, lo] -> [tile, chunk, q, n, hi, lo]
    x = pad.reshape(P // 16, 16, chunks, 2, 4, 4).permute(0, 2, 4, 1, 3, 5)
    return x.reshape(P // 16, chunks, 64, 8).contiguous()


class TalkingWeights:
    def __init__(self, heads: Heads, talk: torch.Tensor, temp: torch.Tensor, rel: torch.Tensor, scale: float,
                 far: float, device):
        """``talk [H, H]``, ``temp [H]``, ``rel [buckets, H]`` as stored (bf16 values)."""
        H = heads.heads
        self.heads = heads
        t64, rows = talk.to(device).double(), rel.shape[0]
        self.sc = (temp.to(device).double() * scale * LOG2E).float().contiguous()
        # every distance from the last bucket's first one on has its bias
        b = buckets(rows, far, math.ceil(far) + 1)
        nfar = int(np.argmax(b == rows - 1)) if (b == rows - 1).any() else len(b) - 1
        self.nfar = nfar
        mixed = (rel.to(device).double()[torch.from_numpy(b[:nfar + 1]).to(device)] @ t64.T * LOG2E).float()

        def table(order):
            out = torch.zeros((nfar + 1, len(order)), dtype=torch.float32, device=device)
            have = [i for i, h in enumerate(order) if h >= 0]
            out[:, have] = mixed[:, [order[i] for i in have]]
            return out

        plain = list(range(H)) + [-1] * ((16 if H <= 16 else 32 if H <= 32 else (H + 63) // 64 * 64) - H)
        self.bias = table(plain)
        if heads.mfma:
            tb = talk.to(device).to(torch.bfloat16).to(torch.float16)  # exact down to 2^-14
            self.talk = mix_fragments(tb, plain)
            if heads.tiled:
                order = heads.slot_heads()
                b = table(order)
                self.bias_far = b[-1].clone()
                self.bias_slots = (b - self.bias_far).contiguous()
                self.talk_slots = mix_fragments(tb, order)
        else:
            self.talk = talk.to(device).float().contiguous()


@dataclass
class QueryRows:
    """Query tokens one by one: per token (int32, device) its block-table row and its
    position; ``rows``: its batch row, None when they are the same."""
    n: int
    bt: torch.Tensor
    tok_seq: torch.Tensor
    tok_pos: torch.Tensor
    rows: torch.Tensor | None
    nsplit: int


@dataclass
class QueryTiles:
    """Blocks of up to ``Heads.tile`` consecutive queries over a range of their pages
    (:func:`tile_items`): int32 ``[n, 8]`` (first batch row, block-table row, position of
    the first, queries, first page, end, partial result or -1, 0), and ``merges [m, 4]``
    (first batch row, queries, first part, parts) of the blocks that are split."""
    items: torch.Tensor
    bt: torch.Tensor
    merges: torch.Tensor | None = None
    parts: int = 0


MIN_PAGES = 16  # pages of a part
MAX_PARTS = 64  # parts that one merge takes


def tile_items(portions, tile: int) -> tuple[np.ndarray, np.ndarray]:
    """Items and merges of ``portions`` (first batch row, block-table row, position,
    tokens). Blocks with more than 1.2 even shares of all pages are split, so that a long
    prompt's last blocks do not outlast the others (a part costs a merge): evenly where
    all items run at once,
    else into such parts and a rest, which fill up the last round; the longest first."""
    b = np.array([(r + j, s, p + j, min(tile, n - j)) for r, s, p, n in portions for j in range(0, n, tile)], np.int64)
    pages = (b[:, 2] + b[:, 3] - 1) // PAGE + 1
    share = max(MIN_PAGES, -(-6 * int(pages.sum()) // (5 * CUS))) if len(b) < 2 * CUS else int(pages.max())
    cap = np.maximum(share, -(-pages // MAX_PARTS))
    parts = -(-pages // cap)
    split = parts > 1
    at = np.repeat(np.arange(len(b)), parts)
    k = np.arange(len(at)) - np.repeat(np.cumsum(parts) - parts, parts)
    if len(at) <= CUS:
        first, end = pages[at] * k // parts[at], pages[at] * (k + 1) // parts[at]
    else:
        first, end = k * cap[at], np.minimum((k + 1) * cap[at], pages[at])
    part0 = np.cumsum(np.where(split, parts, 0)) - np.where(split, parts, 0)
    part = np.where(split[at], part0[at] + k, -1)
    items = np.concatenate([b[at], np.stack([first, end, part, np.zeros_like(k)], 1)], 1)
    merges = np.stack([b[:, 0], b[:, 3], part0, parts], 1)[split]
    return items[np.argsort(first - end, kind="stable")], merges


def split_count(n: int, max_pages: int) -> int:
    """Context splits of the rows kernel: two workgroups of four waves per CU, at least
    a page per wave."""
    return max(1, min(2 * CUS // max(1, n), -(-max_pages // 4), 64))


class Rotary:
    """Rotary positions of the pairs (0, 1), (2, 3), .. of each head's first ``dims`` dims:
    the pair i turns by ``position * base ** (-2 i / dims)``. ``table`` fp32 ``[positions,
    dims padded to 8]``: cos and sin of each pair."""

    def __init__(self, dims: int, base: float, positions: int, device):
        p = torch.arange(positions, dtype=torch.float64)[:, None]
        a = p * base ** (-torch.arange(0, dims, 2, dtype=torch.float64) / dims)
        t = torch.stack([a.cos(), a.sin()], -1).reshape(positions, dims)
        if dims % 8:  # the pad's pairs stay as they are
            t = torch.cat([t, torch.tensor([1.0, 0.0], dtype=torch.float64).repeat(positions, (8 - dims % 8) // 2)], 1)
        self.table = t.float().to(device).contiguous()


@dataclass
class HeadNorm:
    """RMS norm of every head's (and map's) q and k over its ``dim`` values, times ``wq`` /
    ``wk`` (fp32, zero-padded to the head's columns)."""
    wq: torch.Tensor
    wk: torch.Tensor
    dim: int
    eps: float


@dataclass(frozen=True)
class Temperature:
    """q at position p times ``1 + coef ln(floor((p + 1) / every) + 1)``."""
    coef: float
    every: int


def write_kv(z: torch.Tensor, bias: torch.Tensor | None, pages: torch.Tensor, slots: torch.Tensor, h: Heads, ok: int,
             ov: int, rotary: Rotary | None = None, pos: torch.Tensor | None = None, norm: HeadNorm | None = None,
             temperature: Temperature | None = None) -> None:
    """``z [T, >=]`` holds q (columns 0 ..), k (``ok`` ..) and v (``ov`` ..), heads padded.
    Adds the biases (``bias``: q, k, v one after another, or None): q in place, k and v into
    ``pages`` at ``slots`` (-1: dropped). ``norm``: q and k normed per head and map; ``rotary``:
    turned by the rows' ``pos`` (int32 ``[T]``); ``temperature``: q scaled by position."""
    T, nq, nk, nv = z.shape[0], h.heads * h.dkp, h.kv_heads * h.dkp, h.kv_heads * h.dvp
    if pages.dtype != z.dtype or not pages.is_contiguous() or pages.shape[1:] != (h.kv_heads, PAGE * (h.dkp + h.dvp)):
        raise ValueError(f"pages {tuple(pages.shape)} {pages.dtype} do not fit {h}")
    turn, seg = (0, 0, 0, 0), h.dkp // h.maps
    if rotary is not None or temperature is not None:
        if pos is None or pos.dtype != torch.int32 or not pos.is_contiguous() or pos.shape[0] != T:
            raise ValueError("positions of the rows must be contiguous int32")
        turn = (0, pos.data_ptr(), 0, 0) if rotary is None else (rotary.table.data_ptr(), pos.data_ptr(), *rotary.table.shape)
    normed = (0, 0, seg, seg, 0.0) if norm is None else (_f32(norm.wq, (seg,), "wq"), _f32(norm.wk, (seg,), "wk"), seg,
                                                         norm.dim, float(norm.eps))
    warm = (0.0, 0) if temperature is None else (float(temperature.coef), temperature.every)
    rc = _lib.lib().kgs_talking_write(_act(z, T, max(nq, ok + nk, ov + nv), z.dtype, "z"), z.stride(0),
                                      0 if bias is None else _f32(bias, (nq + nk + nv,), "bias"), pages.data_ptr(), slots.data_ptr(), T, nq,
                                      h.kv_heads, h.dkp, h.dvp, ok, ov, *turn, *normed, *warm, int(z.dtype == torch.float32),
                                      _lib.stream_handle(z.device))
    _lib.check(rc, f"talking_write[{T}]")


def attention_rows(q: torch.Tensor, pages: torch.Tensor, w: TalkingWeights, r: QueryRows, out: torch.Tensor) -> torch.Tensor:
    """Attention of single query tokens over their sequences' pages up to their
    positions; ``q [T, >= H dkp]``, ``out [T, >= H dvp]``."""
    h, L = w.heads, _lib.lib()
    f32 = q.dtype == torch.float32
    po = pml = None
    ns = r.nsplit if h.mfma else 1
    if ns > 1:
        po = torch.empty((r.n, ns, h.heads, h.dvp), dtype=torch.float32, device=q.device)
        pml = torch.empty((r.n, ns, h.heads, 2), dtype=torch.float32, device=q.device)
    rc = L.kgs_talking_rows(_act(q, q.shape[0], h.heads * h.dkp, pages.dtype, "q"), q.stride(0), pages.data_ptr(),
                            _act(out, out.shape[0], h.heads * h.dvp, pages.dtype, "out"), out.stride(0), r.bt.data_ptr(),
                            r.bt.shape[1], r.tok_seq.data_ptr(), r.tok_pos.data_ptr(),
                            0 if r.rows is None else r.rows.data_ptr(), 0 if po is None else po.data_ptr(),
                            0 if pml is None else pml.data_ptr(), w.sc.data_ptr(), w.talk.data_ptr(), w.bias.data_ptr(),
                            w.bias.shape[1], w.nfar, r.n, h.heads, h.kv_heads, h.dkp, h.dvp, ns, int(not h.mfma),
                            int(f32), _lib.stream_handle(q.device))
    _lib.check(rc, f"talking_rows[{r.n}x{h.heads}/{ns}]")
    return out


def attention_tiles(q: torch.Tensor, pages: torch.Tensor, w: TalkingWeights, t: QueryTiles, out: torch.Tensor) -> torch.Tensor:
    """Attention of prompt portions (:class:`QueryTiles`), as :func:`attention_rows`."""
    h = w.heads
    if not h.tiled:
        raise ValueError(f"{h} has no tiled kernel")
    if t.items.dtype != torch.int32 or t.items.dim() != 2 or t.items.shape[1] != 8 or not t.items.is_contiguous():
        raise ValueError("items must be contiguous int32 [n, 8]")
    m, po, pml = 0 if t.merges is None else t.merges.shape[0], None, None
    if m:
        po = torch.empty((t.parts * h.tile, h.heads, h.dvp), dtype=torch.float32, device=q.device)
        pml = torch.empty((t.parts * h.tile, h.heads, 2), dtype=torch.float32, device=q.device)
    n = t.items.shape[0]
    scratch = torch.empty((n, h.tile_bytes), dtype=torch.uint8, device=q.device)
    rc = _lib.lib().kgs_talking_tiles(_act(q, q.shape[0], h.heads * h.dkp, torch.bfloat16, "q"), q.stride(0),
                                      pages.data_ptr(), _act(out, out.shape[0], h.heads * h.dvp, torch.bfloat16, "out"),
                                      out.stride(0), t.bt.data_ptr(), t.bt.shape[1], t.items.data_ptr(),
                                      n, t.merges.data_ptr() if m else 0, m, po.data_ptr() if m else 0,
                                      pml.data_ptr() if m else 0, scratch.data_ptr(), w.sc.data_ptr(), w.talk_slots.data_ptr(),
                                      w.bias_slots.data_ptr(), w.bias_far.data_ptr(), w.bias_slots.shape[1], w.nfar, h.heads, h.kv_heads,
                                      h.dkp, h.dvp, _lib.stream_handle(q.device))
    _lib.check(rc, f"talking_tiles[{n}x{h.heads}]")
    return out
