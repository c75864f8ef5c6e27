"""Mixture of experts (``native/kernels/moe.hip``): router, sorted order, grouped GEMMs.

:func:`route` picks every token's experts; :func:`plan` sorts the choices by expert;
:func:`gate_up` and :func:`down` run the experts over the sorted rows. Nothing comes
back to the host, so a step of fixed shape can be captured in a hipGraph.
"""
from __future__ import annotations

from dataclasses import dataclass

import torch

from . import _lib
from .activation import Gate
from .decode import CUS
from .hyper import _act, _f32

MAX_EXPERTS = 1024


@dataclass
class Choices:
    ids: torch.Tensor      # [T, top] int32, -1: a padding row's
    rank: torch.Tensor     # [T, top] rank among the tokens of the expert
    weight: torch.Tensor   # [T, top] fp32
    counts: torch.Tensor   # [E] tokens of every expert


@dataclass
class Plan:
    pos: torch.Tensor      # [T, top] sorted row of each choice, -1: none
    rows: torch.Tensor     # [T * top] token of each sorted row
    weight: torch.Tensor   # [T * top] its weight
    tiles: torch.Tensor    # [max_tiles, 4] (expert, first row, rows, 0)
    ntiles: torch.Tensor
    max_tiles: int
    bm: int


def tile_rows(T: int, top: int, experts: int, dtype) -> int:
    """Rows of a GEMM tile: the high one where the experts' shares fill it."""
    if dtype == torch.float32:
        return 64
    return 256 if T * top >= 192 * experts else 128


def router_rows(n: int) -> int:
    """Router rows padded to a size the MFMA router has (above 64: any multiple of 16)."""
    return next((s for s in (16, 32, 64) if s >= n), (n + 15) // 16 * 16)


def route(h: torch.Tensor, w: torch.Tensor, counts: torch.Tensor, top: int, slots: torch.Tensor | None = None) -> Choices:
    """``w [ep, wp]``: the router, rows padded to a multiple of 16. ``counts [E]`` must
    be zero. Rows whose slot is negative choose nothing."""
    T, E = h.shape[0], counts.shape[0]
    ep, wp = w.shape
    if w.dtype != h.dtype or not w.is_contiguous() or counts.dtype != torch.int32 or E > MAX_EXPERTS:
        raise ValueError("router weights must be contiguous and of h's dtype, counts int32")
    mk = lambda dt: torch.empty((T, top), dtype=dt, device=h.device)  # noqa: E731
    c = Choices(mk(torch.int32), mk(torch.int32), mk(torch.float32), counts)
    rc = _lib.lib().kgs_moe_route(_act(h, T, wp, w.dtype, "h"), h.stride(0), w.data_ptr(),
                                  0 if slots is None else slots.data_ptr(), counts.data_ptr(), c.ids.data_ptr(),
                                  c.rank.data_ptr(), c.weight.data_ptr(), T, E, ep, wp, top,
                                  int(h.dtype == torch.float32), _lib.stream_handle(h.device))
    _lib.check(rc, f"moe_route[{T}x{E}]")
    return c


@dataclass(frozen=True)
class Softmax:
    """Routing by softmax scores over ``experts`` and ``identity`` outputs that return
    their input: the ``top`` largest of score + correction among the best ``keep`` of
    ``groups`` groups of neighbours (a group counts as its largest), with their scores,
    normalised, times ``scale`` as weights."""
    experts: int
    identity: int
    top: int
    groups: int
    keep: int
    scale: float


def route_softmax(h: torch.Tensor, w: torch.Tensor, counts: torch.Tensor, r: Softmax, correction: torch.Tensor,
                  slots: torch.Tensor | None = None, gate: bool = False
                  ) -> tuple[Choices, torch.Tensor | None, torch.Tensor | None]:
    """As :func:`route` with the other choice; the choices' weights scale the experts'
    outputs. Also, fp32 ``[T]``: the weights of a token's identity outputs together (None
    without any) and, with ``gate``, the sigmoid of the router row after the outputs."""
    T, E, n = h.shape[0], counts.shape[0], r.experts + r.identity
    ep, wp = w.shape
    if w.dtype != h.dtype or not w.is_contiguous() or counts.dtype != torch.int32 or E != r.experts or n > MAX_EXPERTS:
        raise ValueError("router weights must be contiguous and of h's dtype, counts int32, one per expert")
    mk = lambda dt, *s: torch.empty((T, *s), dtype=dt, device=h.device)  # noqa: E731
    c = Choices(mk(torch.int32, r.top), mk(torch.int32, r.top), mk(torch.float32, r.top), counts)
    ident, g = mk(torch.float32) if r.identity else None, mk(torch.float32) if gate else None
    rc = _lib.lib().kgs_moe_route_softmax(_act(h, T, wp, w.dtype, "h"), h.stride(0), w.data_ptr(),
                                          0 if slots is None else slots.data_ptr(), counts.data_ptr(), c.ids.data_ptr(),
                                          c.rank.data_ptr(), c.weight.data_ptr(), _f32(correction, (n,), "correction"),
                                          0 if ident is None else ident.data_ptr(), 0 if g is None else g.data_ptr(), T, E,
                                          r.identity, r.groups, r.keep, float(r.scale), ep, wp, r.top,
                                          int(h.dtype == torch.float32), _lib.stream_handle(h.device))
    _lib.check(rc, f"moe_route_softmax[{T}x{n}]")
    return c, ident, g


def plan(c: Choices, bm: int) -> Plan:
    T, top = c.ids.shape
    E, n = c.counts.shape[0], T * top
    # every expert can end in one partly filled tile, but not more of them than rows
    most = min(n, n // bm + min(E, n))
    i32 = lambda *s: torch.empty(s, dtype=torch.int32, device=c.ids.device)  # noqa: E731
    p = Plan(i32(T, top), i32(n), torch.empty(n, dtype=torch.float32, device=c.ids.device), i32(most, 4), i32(1), most, bm)
    rc = _lib.lib().kgs_moe_plan(c.counts.data_ptr(), c.ids.data_ptr(), c.rank.data_ptr(), c.weight.data_ptr(),
                                 p.pos.data_ptr(), p.rows.data_ptr(), p.weight.data_ptr(), p.tiles.data_ptr(),
                                 p.ntiles.data_ptr(), T, top, E, bm, _lib.stream_handle(c.ids.device))
    _lib.check(rc, f"moe_plan[{n}x{E}]")
    return p


def _grouped(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor, p: Plan, T: int, nslice: int,
             gate: Gate | None) -> torch.Tensor:
    E, N, K = w.shape
    if a.dtype != w.dtype or not w.is_contiguous():
        raise ValueError("activations and expert weights must share a dtype, weights contiguous")
    rc = _lib.lib().kgs_moe_grouped(_act(a, a.shape[0], K, w.dtype, "a"), a.stride(0), w.data_ptr(), out.data_ptr(),
                                    out.stride(-2), p.rows.data_ptr(), p.weight.data_ptr(), p.tiles.data_ptr(),
                                    p.ntiles.data_ptr(), p.max_tiles, p.bm, T, p.rows.shape[0], N, K, nslice,
                                    gate.limit if gate else 0.0, GATES[gate.act] if gate else 0, int(gate is not None),
                                    int(w.dtype == torch.float32), _lib.stream_handle(a.device))
    _lib.check(rc, f"moe_grouped[{p.rows.shape[0]}x{E}x{N}x{K}/{nslice}]")
    return out


GATES = {"clamped": 0, "silu": 1}


def gate_up(h: torch.Tensor, w: torch.Tensor, p: Plan, gate: Gate) -> torch.Tensor:
    """``[P, ff]``: the gated product of each sorted row, ``w [E, 2 ff, K]``. ``clamped``:
    of its weighted input; ``silu``: times its weight, which so scales the expert's output."""
    out = torch.empty((p.rows.shape[0], w.shape[1] // 2), dtype=h.dtype, device=h.device)
    return _grouped(h, w, out, p, h.shape[0], 1, gate)


def split_k(p: Plan, N: int, K: int) -> int:
    """K slices of the down projection: more workgroups where a few tokens' tiles leave
    CUs without one."""
    ns = 1
    while p.bm == 128 and ns < 4 and 2 * ns * p.max_tiles * (N // 128) <= CUS and K % (256 * ns) == 0:
        ns *= 2
    return ns


def down(a: torch.Tensor, w: torch.Tensor, p: Plan) -> torch.Tensor:
    """``w[expert] @ a`` per sorted row: ``[P, N]``, or fp32 partial products
    ``[slices, P, N]`` (summed by :func:`kgs.ops.residual.residual_add`)."""
    E, N, K = w.shape
    ns = 1 if a.dtype == torch.float32 else split_k(p, N, K)
    P = p.rows.shape[0]
    out = (torch.empty((P, N), dtype=a.dtype, device=a.device) if ns == 1 else
           torch.empty((ns, P, N), dtype=torch.float32, device=a.device))
    return _grouped(a, w, out, p, P, ns, None)
