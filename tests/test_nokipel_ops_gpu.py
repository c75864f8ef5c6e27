"""Nokipel's kernels one by one against plain references: norm by parts and everything the
residual adds, clamped gates, group-limited routing with identity experts, rotary positions
and the cache write, chunked attention (rows, tiles, plain), lightning attention (steps,
chunks, segments) -- with inputs that stand out where a fault would hide."""
import os
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

from oracles import nokipel as O  # noqa: E402

pytestmark = pytest.mark.gpu
BF, F32 = torch.bfloat16, torch.float32


def rnd(*shape, seed=0, scale=1.0, dtype=F32):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def rel_err(got, want):
    got, want = got.detach().cpu().double(), want.double()
    assert got.shape == want.shape
    return float((got - want).abs().max() / want.abs().max())


def i32(a):
    return torch.tensor(np.asarray(a), dtype=torch.int32).cuda()


# ------------------------------------------------------------------- residual
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width,wp,groups,T", [(140, 256, 5, 4), (240, 256, 1, 3), (1200, 1280, 6, 3), (2048, 2048, 8, 3),
                                               (100, 256, 100, 2), (5120, 5120, 64, 2), (16384, 16384, 2, 2)])
def test_residual_and_norm_by_parts(dtype, width, wp, groups, T):
    """Every input of the residual, alone and together, for parts that are a multiple of
    eight columns or not; parts differ in size, so a norm over the row would show."""
    from kgs.ops.residual import Embedding, ExpertRows, Norm, Scaled, residual_add, residual_embed

    pad = lambda t: torch.nn.functional.pad(t, (0, wp - width))  # noqa: E731
    loud = torch.repeat_interleave(4.0 ** torch.arange(groups).remainder(4), width // groups)
    emb = pad((rnd(11, width, seed=1) * loud).to(dtype))
    w, w2 = pad(1 + rnd(width, seed=2, scale=0.3)), pad(1 + rnd(width, seed=3, scale=0.3))
    toks = torch.tensor([(3 * i + 1) % 11 for i in range(T)], dtype=torch.int32)
    norm = Norm(width, 1e-3, groups, 0.0)
    x, h = residual_embed(toks.cuda(), emb.cuda(), 0.75, w.cuda(), norm)
    e = 0.75 * emb[toks.long()].double()
    tol = 3e-6 if dtype == F32 else 5e-3

    def normed(s, w):
        return O.group_norm(s[:, :width], w[:width].double(), groups, 1e-3)

    assert rel_err(x, e) < 1e-6 and rel_err(h[:, :width], normed(e, w)) < tol and (h[:, width:] == 0).all()
    a, b0, b1 = (pad(rnd(T, width, seed=s, dtype=dtype)) for s in (4, 5, 6))
    s0, s1 = rnd(T, seed=7), rnd(T, seed=8)
    y = pad(rnd(2 * T, width, seed=9, dtype=dtype))
    pos = torch.tensor([[(3 * t + j) % (2 * T) if (t + j) % 3 else -1 for j in range(3)] for t in range(T)], dtype=torch.int32)
    rows = torch.stack([sum((y[p].double() for p in r if p >= 0), torch.zeros(wp, dtype=torch.float64)) for r in pos.tolist()])
    for on in ("a", "y", "0", "01", "e", "a01ye"):
        x2 = x.clone()
        h = residual_add(x2, a.cuda() if "a" in on else None, None, ExpertRows(y.cuda(), pos.cuda()) if "y" in on else None,
                         w2.cuda(), norm, dtype,
                         scaled=[Scaled(b.cuda(), s.cuda()) for c, b, s in (("0", b0, s0), ("1", b1, s1)) if c in on],
                         embedding=Embedding(toks.cuda(), emb.cuda(), 0.75) if "e" in on else None)
        s = e + ("a" in on) * a.double() + ("y" in on) * rows + ("0" in on) * s0.double()[:, None] * b0.double() + \
            ("1" in on) * s1.double()[:, None] * b1.double() + ("e" in on) * e
        assert rel_err(x2, s) < 1e-6, on
        assert rel_err(h[:, :width], normed(s, w2)) < tol, on


# --------------------------------------------------------------- feed-forward
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("T,K,ff,limit", [(1, 256, 128, 1.0), (5, 512, 192, 0.6), (33, 512, 512, 2.0), (130, 256, 320, 1.0),
                                          (600, 512, 576, 0.7), (2048, 512, 8192, 1.5), (512, 512, 512, 1.0)])
def test_clamped_gate(T, K, ff, limit, dtype):
    """Every kernel form of the fused gate and up projections, inputs on both sides of
    the clamps."""
    from kgs.ops.activation import Gate
    from kgs.ops.linear import Projection

    x, gate, up = rnd(T, K, seed=T, dtype=dtype), rnd(ff, K, seed=1, scale=1.5 * K ** -0.5, dtype=dtype), \
        rnd(ff, K, seed=2, scale=1.5 * K ** -0.5, dtype=dtype)
    p = Projection(torch.cat([gate, up]).cuda(), gated=Gate("clamped", limit))
    sel = range(0, T, max(1, T // 100))
    xd = x[list(sel)].double()
    eye = {"gate": gate.double(), "up": up.double(), "down": torch.eye(ff, dtype=torch.float64)}
    want = O.dense(xd, eye, "", limit)
    got = p(x.cuda())[list(sel)]
    assert rel_err(got, want) < (1e-5 if dtype == F32 else 1e-2)


ROUTE = [  # tokens, experts, identity, top, groups, keep, width, gate
    (1, 4, 0, 1, 1, 1, 256, False), (7, 5, 1, 2, 3, 2, 256, True), (65, 14, 2, 3, 4, 1, 512, True),
    (300, 20, 4, 6, 6, 3, 256, False), (33, 120, 8, 8, 16, 2, 256, True), (40, 1, 1, 2, 1, 1, 256, True),
    (19, 60, 3, 5, 7, 7, 512, True)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("T,E,ident,top,groups,keep,W,gate", ROUTE)
def test_routing(T, E, ident, top, groups, keep, W, gate, dtype):
    """Choices, weights, identity shares, counts and the shared gate; corrections large
    enough that choice scores are negative and weights taken with them would show."""
    from kgs.ops import moe as M

    n = E + ident
    h, w = rnd(T, W, seed=T, dtype=dtype), rnd(n + gate, W, seed=1, scale=2 * W ** -0.5, dtype=dtype)
    corr = rnd(n, seed=2, scale=0.3)
    slots = torch.arange(T, dtype=torch.int32)
    slots[3::7] = -1
    real = slots >= 0
    counts = torch.zeros(E, dtype=torch.int32, device="cuda")
    r = M.Softmax(E, ident, top, groups, keep, 1.7)
    wp = torch.nn.functional.pad(w, (0, 0, 0, M.router_rows(n + gate) - n - gate)).cuda()
    c, idw, g = M.route_softmax(h.cuda(), wp, counts, r, corr.cuda(), slots.cuda(), gate=gate)
    cfg = {"top": top, "scale": 1.7, "groups": {"count": groups, "keep": keep}}
    idx, wt = O.route(h.double(), w[:n].double(), corr.double(), cfg)
    ids, weight = c.ids.cpu(), c.weight.cpu().double()
    for t in range(T):
        got = {int(e): float(x) for e, x in zip(ids[t], weight[t]) if e >= 0}
        want = {int(e): float(x) for e, x in zip(idx[t], wt[t]) if e < E} if real[t] else {}
        assert got.keys() == want.keys(), t
        assert all(abs(got[e] - want[e]) < 1e-5 for e in got), t
        if ident:
            share = float(wt[t][idx[t] >= E].sum()) if real[t] else 0.0
            assert abs(float(idw[t]) - share) < 1e-5
    assert (idw is None) == (ident == 0)
    assert counts.cpu().tolist() == [int((ids == e).sum()) for e in range(E)]
    if gate:
        assert rel_err(g, torch.sigmoid(h.double() @ w[n].double())) < 1e-5
    # the sorted order and the experts' products
    ff = 128
    gu, dn = rnd(E, 2 * ff, W, seed=3, scale=W ** -0.5, dtype=dtype), rnd(E, 256, ff, seed=4, scale=ff ** -0.5, dtype=dtype)
    from kgs.ops.activation import Gate

    p = M.plan(c, M.tile_rows(T, top, E, dtype))
    y = M.down(M.gate_up(h.cuda(), gu.cuda(), p, Gate("silu")), dn.cuda(), p)
    y = (y.sum(0) if y.dim() == 3 else y).cpu().double()
    pos = p.pos.cpu()
    assert sorted(pos[pos >= 0].tolist()) == list(range(int((ids >= 0).sum()))) and ((pos >= 0) == (ids >= 0)).all()
    got, want = [], []
    for t in range(0, T, max(1, T // 40)):
        for j in range(top):
            e = int(ids[t, j])
            if e >= 0:
                we = {"gate": gu[e, :ff].double(), "up": gu[e, ff:].double(), "down": dn[e].double()}
                got.append(y[pos[t, j]])
                want.append(weight[t, j] * O.expert(h[t].double(), we, ""))
    if got:
        assert rel_err(torch.stack(got), torch.stack(want)) < (1e-5 if dtype == F32 else 2e-2)


def test_groups_are_chosen_by_their_largest_and_may_be_negative():
    """All choice scores below zero: an excluded group must not win with a 0, and a group
    of many middling experts loses against one with a single better one."""
    from kgs.ops import moe as M

    h = torch.ones(1, 256, dtype=BF)
    w = torch.zeros(16, 256, dtype=BF)
    corr = torch.tensor([-3.0, -3.0, -3.0, -2.0, -4.0, -9.0, -2.5, -2.5, -2.5])  # groups of 3: best -3, -2, -2.5
    counts = torch.zeros(9, dtype=torch.int32, device="cuda")
    c, _, _ = M.route_softmax(h.cuda(), w.cuda(), counts, M.Softmax(9, 0, 3, 3, 1, 2.0), corr.cuda())
    assert sorted(c.ids.cpu()[0].tolist()) == [3, 4, 5]
    assert torch.allclose(c.weight.cpu(), torch.full((1, 3), 2 / 3), atol=1e-6)


# ------------------------------------------------------------------- attention
class Case:
    """Sequences with scattered pages, keys and values written by the product's own write."""

    def __init__(self, shape, lens, dtype, chunk, rot=None, seed=0, sharp=()):
        from kgs.ops.paged import paged_heads
        from kgs.ops.talking import HeadPages, Rotary, write_kv

        H, G, d, dv = shape
        self.lens, self.dtype, self.chunk = lens, dtype, chunk
        self.h = h = paged_heads(H, G, d, dv, dtype)
        T = sum(lens)
        self.scale = 1.3 * d ** -0.5
        q, k, v = rnd(T, H, d, seed=seed), rnd(T, G, d, seed=seed + 1), rnd(T, G, dv, seed=seed + 2)
        for i, j, f in sharp:  # query i of the first sequence finds key j by far the best
            k[j] *= 0.3
            for x in range(H):
                q[i, x] = f * 12 * k[j, x // (H // G)] / k[j, x // (H // G)].norm()
            k[j] *= 5
        q, k, v = (t.to(dtype) for t in (q, k, v))
        b = {n: rnd(c, seed=seed + s, scale=0.2).to(BF).float() for n, c, s in (("q", H * d, 3), ("k", G * d, 4), ("v", G * dv, 5))}
        cat = lambda t, n, dp, s: torch.nn.functional.pad(t, (0, dp - s)).reshape(*t.shape[:-2], n * dp)  # noqa: E731
        offs = [0, -(-H * h.dkp // 64) * 64]
        offs.append(offs[1] + -(-G * h.dkp // 64) * 64)
        z = torch.zeros(T, offs[2] + G * h.dvp + 64, dtype=dtype)
        z[:, :H * h.dkp] = cat(q, H, h.dkp, d)
        z[:, offs[1]:offs[1] + G * h.dkp] = cat(k, G, h.dkp, d)
        z[:, offs[2]:offs[2] + G * h.dvp] = cat(v, G, h.dvp, dv)
        bias = torch.cat([cat(b["q"].reshape(H, d), H, h.dkp, d), cat(b["k"].reshape(G, d), G, h.dkp, d),
                          cat(b["v"].reshape(G, dv), G, h.dvp, dv)])
        per = [-(-n // 32) for n in lens]
        perm = np.random.default_rng(seed).permutation(sum(per)) + 1
        self.bt = np.zeros((len(lens), max(per)), np.int64)
        slots, pos, at = [], [], 0
        for s, n in enumerate(lens):
            self.bt[s, :per[s]] = perm[at:at + per[s]]
            at += per[s]
            slots += [self.bt[s, p // 32] * 32 + p % 32 for p in range(n)]
            pos += list(range(n))
        self.pages = HeadPages({0: h}, sum(per) + 1, dtype, "cuda").pages[0]
        self.pages[0] = 1e4  # never read
        self.z = z.cuda()
        rotary = None if rot is None else Rotary(*rot, max(lens), "cuda")
        write_kv(self.z, bias.cuda(), self.pages, i32(slots), h, offs[1], offs[2], rotary, i32(pos))
        base = np.cumsum([0] + lens)
        self.want = []
        for s in range(len(lens)):
            sl = slice(base[s], base[s + 1])
            qs, ks, vs = (t[sl].double() + b[n].double().reshape(t.shape[1:]) for t, n in ((q, "q"), (k, "k"), (v, "v")))
            if rot is not None:
                qs, ks = O.rotate(qs, *rot), O.rotate(ks, *rot)
            mask = O.chunk_mask(lens[s], chunk or 1 << 30)
            o = [torch.softmax((qs[:, x] @ ks[:, x // (H // G)].T * self.scale).masked_fill(~mask, -torch.inf), -1)
                 @ vs[:, x // (H // G)] for x in range(H)]
            self.want.append(torch.stack(o, 1))
        self.dv = dv

    def out(self):
        return torch.full((sum(self.lens), self.h.heads * self.h.dvp), float("nan"), dtype=self.dtype, device="cuda")

    def rows(self, sel, nsplit):
        from kgs.ops.paged import paged_rows
        from kgs.ops.talking import QueryRows

        base = np.cumsum([0] + self.lens)
        r = QueryRows(len(sel), i32(self.bt), i32([s for s, _ in sel]), i32([p for _, p in sel]),
                      i32([base[s] + p for s, p in sel]), nsplit)
        return paged_rows(self.z, self.pages, self.h, self.scale, self.chunk, r, self.out())

    def tiles(self, portions):
        from kgs.ops.paged import Portions, paged_tiles, portion_items, tile_queries

        base = np.cumsum([0] + self.lens)
        items = portion_items([(base[s] + p, s, p, n) for s, p, n in portions], tile_queries(self.h), self.chunk)
        return paged_tiles(self.z, self.pages, self.h, self.scale, self.chunk, Portions(i32(items), i32(self.bt)), self.out())

    def check(self, got, sel, what):
        base, tol = np.cumsum([0] + self.lens), 2e-5 if self.dtype == F32 else 2e-2
        got = got.cpu().double().reshape(len(got), self.h.heads, self.h.dvp)
        assert int(torch.isfinite(got[:, 0, 0]).sum()) == len(set(sel)), what  # and no other row
        for s, p in sel:
            g, w = got[base[s] + p], self.want[s][p]
            assert (g[:, self.dv:] == 0).all(), (what, s, p)
            err = float((g[:, :self.dv] - w).abs().max()) / float(self.want[s].abs().max())
            assert err < tol, f"{what}: sequence {s} position {p} off by {err:.1e}"


# heads, kv heads, dim, vdim: groups of 1, 3, 4, 16, 20 and 128 heads; sizes the MFMA kernels pad or leave
SHAPES = [(6, 2, 40, 24), (8, 8, 64, 128), (16, 4, 128, 128), (32, 2, 100, 64), (20, 1, 64, 64), (128, 1, 64, 64),
          (6, 3, 160, 80), (2, 1, 16, 300)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("chunk", [0, 1, 17, 48, 64])
@pytest.mark.parametrize("shape", SHAPES, ids=str)
def test_attention(shape, chunk, dtype):
    """Single tokens at page borders, chunk borders and splits, whole prompts and portions
    at any position; rows that were not asked for stay as they were."""
    c = Case(shape, [1, 70, 131, 33], dtype, chunk)
    sel = [(0, 0), (1, 0), (1, 16), (1, 17), (1, 31), (1, 32), (1, 47), (1, 48), (1, 69), (2, 63), (2, 64), (2, 95), (2, 96),
           (2, 130), (3, 32)]
    for nsplit in (1, 2, 5):
        c.check(c.rows(sel, nsplit), sel, f"rows / {nsplit}")
    from kgs.ops.paged import tile_queries

    if tile_queries(c.h):
        portions = [(0, 0, 1), (1, 0, 70), (2, 0, 40), (2, 40, 16), (2, 56, 17), (2, 73, 58), (3, 5, 28)]
        c.check(c.tiles(portions), [(s, p + j) for s, p, n in portions for j in range(n)], "tiles")
    else:
        assert dtype == F32 or shape in SHAPES[6:]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("chunk", [0, 100, 256])
@pytest.mark.parametrize("shape", [(9, 3, 56, 40), (16, 4, 128, 128)], ids=str)
def test_scores_that_stand_out(shape, chunk, dtype):
    """Keys that one query finds by far the best -- a chunk's first, the last before it
    (not seen), at page borders, far back, the query's own."""
    sharp = [(299, 0, 1.0), (290, 256, 2.0), (288, 255, 3.0), (199, 100, 2.5), (198, 99, 3.0), (99, 31, 2.0), (120, 120, 4.0),
             (255, 32, 2.0), (250, 224, 3.0)]
    c = Case(shape, [301], dtype, chunk, sharp=sharp)
    sel = [(0, t) for t, _, _ in sharp]
    c.check(c.rows(sel, 1), sel, "rows")
    c.check(c.rows(sel, 4), sel, "rows / 4")
    from kgs.ops.paged import tile_queries

    if tile_queries(c.h):
        c.check(c.tiles([(0, 0, 301)]), [(0, p) for p in range(301)], "tiles")
        c.check(c.tiles([(0, 110, 191)]), [(0, p) for p in range(110, 301)], "tiles")


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("shape,rot", [((6, 2, 40, 24), (40, 100.0)), ((6, 2, 40, 24), (12, 1e4)), ((4, 4, 64, 64), (2, 10.0)),
                                       ((8, 2, 128, 128), (100, 5e5)), ((2, 1, 160, 32), (64, 1e6))], ids=str)
def test_rotary_positions(shape, rot, dtype):
    """Neighbouring pairs of some or all dimensions; padded dimensions and the rest stay."""
    c = Case(shape, [150, 40], dtype, 70, rot=rot, seed=3)
    sel = [(0, p) for p in (0, 1, 69, 70, 71, 149)] + [(1, 39)]
    c.check(c.rows(sel, 2), sel, "rows")


def test_rotary_table_far_out():
    from kgs.ops.talking import Rotary

    t = Rotary(10, 1e4, 40000, "cpu").table
    assert t.shape == (40000, 16) and torch.equal(t[:, 10:], torch.tensor([1.0, 0.0] * 3).repeat(40000, 1))
    a = 39999 * 1e4 ** (-4 / 10)
    assert abs(float(t[39999, 4]) - np.cos(a)) < 1e-6 and abs(float(t[39999, 5]) - np.sin(a)) < 1e-6


# ------------------------------------------------------------------- lightning
class Lightning:
    def __init__(self, H, K, V, dtype, decay, slots=6):
        from kgs.ops.lightning import Decays, LightningShape, LightningState

        self.sh, self.dtype, self.decay = LightningShape(H, K, V), dtype, decay
        self.state, self.d = LightningState(self.sh, slots, "cuda"), Decays(decay, "cuda")
        self.state.S.fill_(float("nan"))  # position 0 must not read it

    def rows(self, T, seed, scale=1.0):
        s, H = self.sh, self.sh.heads
        return [rnd(T, H, n, seed=seed + i, scale=scale, dtype=self.dtype) for i, n in enumerate((s.dim, s.dim, s.vdim))]

    def run(self, seqs, units=None, split=False):
        """``seqs``: (rows, position, slot); outputs ``[T, H, V]`` per sequence."""
        from kgs.ops.delta import RaggedSeqs
        from kgs.ops.lightning import SegmentPlan, lightning_forward, segment_plan

        s, H = self.sh, self.sh.heads
        n = [len(x[0][0]) for x in seqs]
        row0 = np.cumsum([0] + n[:-1])
        cat = lambda j, p: torch.nn.functional.pad(torch.cat([x[0][j] for x in seqs]), (0, p - seqs[0][0][j].shape[2])).reshape(sum(n), -1)  # noqa: E731
        z = torch.cat([torch.zeros(sum(n), 64, dtype=self.dtype), cat(0, s.kp), cat(1, s.kp), cat(2, s.vp)], 1).cuda()
        offs = (64, 64 + H * s.kp, 64 + 2 * H * s.kp)
        p = segment_plan(n, units or H * s.slabs, self.dtype == BF and s.dim <= 128)
        assert not split or len(p["scans"])
        plan = SegmentPlan(len(p["step"]), i32(p["step"]) if len(p["step"]) else None, i32(p["items"]) if len(p["items"]) else None,
                           i32(p["scans"]) if len(p["scans"]) else None, p["buffers"])
        rs = RaggedSeqs(None, i32(row0), i32(n), i32([x[1] for x in seqs]), i32([x[2] for x in seqs]))
        o = lightning_forward(z, offs, s, self.d, self.state, rs, plan).cpu().reshape(sum(n), H, s.vp)
        assert (o[..., s.vdim:] == 0).all()
        return [o[r:r + k, :, :s.vdim] for r, k in zip(row0, n)]

    def oracle(self, parts):
        q, k, v = (O.silu(torch.cat([p[j] for p in parts]).double()) for j in range(3))
        return O.recurrence(q, k, v, self.decay)


def decays(H):
    return [0.0 if h == 2 else 1.0 if h == 3 else float(1 - 0.6 * 0.35 ** h) for h in range(H)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,K,V", [(5, 24, 40), (4, 64, 128), (2, 128, 64), (3, 100, 200), (1, 1, 1), (2, 200, 72)], ids=str)
def test_lightning(H, K, V, dtype):
    """Portions of every kind beside each other -- steps, one chunk, chunks with a rest,
    a sequence that goes on -- with decays of 0 and 1 among the heads."""
    c = Lightning(H, K, V, dtype, decays(H))
    tol = 1e-5 if dtype == F32 else 1.5e-2
    lens = [1, 16, 2, 64, 15, 150]
    first = [c.rows(n, 10 * i) for i, n in enumerate(lens)]
    got1 = c.run([(r, 0, i) for i, r in enumerate(first)])
    more = [(1, 3), (3, 77), (4, 1), (5, 16), (2, 129)]  # (sequence, tokens)
    second = [c.rows(n, 100 + 10 * i) for i, (_, n) in enumerate(more)]
    got2 = c.run([(r, lens[s], s) for r, (s, _) in zip(second, more)])
    for i, n in enumerate(lens):
        parts = [first[i]] + [r for r, (s, _) in zip(second, more) if s == i]
        got = torch.cat([got1[i]] + [g for g, (s, _) in zip(got2, more) if s == i])
        want = c.oracle(parts)
        for h in range(H):
            assert rel_err(got[:, h], want[:, h]) < tol, (i, n, h)


@pytest.mark.parametrize("H,K,V", [(2, 64, 64), (3, 128, 256), (1, 32, 128)], ids=str)
def test_lightning_segments(H, K, V):
    """A long portion cut into segments that run side by side, from a state and from
    none, beside short ones; the token after it steps from the state it left."""
    c = Lightning(H, K, V, BF, [0.999, 0.9, 0.995][:H])
    a, b, s = c.rows(70, 1), c.rows(1500, 2), c.rows(5, 3)
    x = c.rows(700, 4)
    one = c.run([(a, 0, 1), (x, 0, 2)])
    two = c.run([(s, 0, 3), (b, 70, 1), (x, 0, 4)], split=True)
    tail = c.rows(3, 5)
    three = c.run([(tail, 1570, 1), (tail, 700, 4), (tail, 700, 2)])
    want = c.oracle([a, b, tail])
    assert rel_err(torch.cat([one[0], two[1], three[0]]), want) < 1.5e-2
    want = c.oracle([x, tail])
    assert rel_err(torch.cat([two[2], three[1]]), want) < 1.5e-2
    assert rel_err(torch.cat([one[1], three[2]]), want) < 1.5e-2
    assert rel_err(two[0], c.oracle([s])) < 1e-5


def test_lightning_reads_a_far_key():
    """One key early in the sequence that only the last query matches: its value must
    come through the state, across chunks and segments, at its decay."""
    for dtype, units in ((F32, None), (BF, None), (BF, 100000)):
        c = Lightning(1, 64, 64, dtype, [0.9995])
        q, k, v = c.rows(900, 1, scale=0.01)
        q[:], k[:] = -30, -30            # silu: zero
        k[5, 0, 7], v[5, 0] = 8, 4
        q[899, 0, 7] = 8
        o = c.run([([q, k, v], 0, 0)], units=units)[0]
        want = c.oracle([[q, k, v]])
        assert rel_err(o[899], want[899]) < (5e-5 if dtype == F32 else 4e-3) and float(o[:899].abs().max()) < 1e-6


def test_lightning_state_is_32_bit():
    """Small contributions on top of a large one, for a thousand tokens: a state held in
    fewer bits would lose them."""
    for dtype in (F32, BF):
        c = Lightning(1, 64, 64, dtype, [1.0])
        q, k, v = c.rows(1000, 1)
        k[:], v[:], q[:] = 4, 0.01, 4
        v[0] = 100
        o = c.run([([q, k, v], 0, 0)])[0]
        assert rel_err(o - o[0], c.oracle([[q, k, v]]) - c.oracle([[q, k, v]])[0]) < (2e-3 if dtype == F32 else 1e-2), dtype


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,V,vp,ld", [(3, 40, 64, 192), (1, 64, 64, 64), (8, 128, 128, 1024), (32, 100, 128, 4096), (60, 200, 256, 15360)])
def test_lightning_out(H, V, vp, ld, dtype):
    from kgs.ops.lightning import lightning_out

    T, n = 5, H * vp
    pad = lambda t: torch.nn.functional.pad(t, (0, vp - V)).reshape(*t.shape[:-2], n)  # noqa: E731
    o, w, g = rnd(T, H, V, seed=1) * (1 + torch.arange(H))[:, None], 1 + rnd(H, V, seed=2, scale=0.2), rnd(T, H, V, seed=3, dtype=dtype)
    y = lightning_out(pad(o).cuda(), pad(w).cuda(), pad(g).cuda(), H * V, 0.01, ld)
    want = O.rms(o.double().reshape(T, -1), 0.01) * w.double().reshape(-1) * torch.sigmoid(g.double().reshape(T, -1))
    got = y[:, :n].cpu().reshape(T, H, vp)
    assert rel_err(got[..., :V].reshape(T, -1), want) < (2e-6 if dtype == F32 else 6e-3)
    assert (got[..., V:] == 0).all() and (y[:, n:] == 0).all()
