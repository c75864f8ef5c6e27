"""Nufusun's kernels one by one against plain references: residual and norm, routing,
sorted order and grouped products, biases and cache write, talking-heads attention
(rows, tiles, plain) with scores that stand out where a fault would hide."""
import os
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

from oracles import nufusun as O  # noqa: E402

pytestmark = pytest.mark.gpu
BF, F32 = torch.bfloat16, torch.float32


def rnd(*shape, seed=0, scale=1.0, dtype=F32):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def rel_err(got, want):
    got, want = got.detach().cpu().double(), want.double()
    return float((got - want).abs().max() / want.abs().max())


# ------------------------------------------------------------------- residual
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width,wp,T", [(140, 256, 5), (2048, 2048, 3), (5000, 5120, 2), (16384, 16384, 2)])
def test_residual(dtype, width, wp, T):
    from kgs.ops.residual import ExpertRows, Norm, residual_add, residual_embed

    pad = lambda t: torch.nn.functional.pad(t, (0, wp - width))  # noqa: E731
    emb = pad(rnd(11, width, seed=1, dtype=dtype))
    w, w2, ab = (pad(rnd(width, seed=s, scale=0.3)) for s in (2, 3, 4))
    toks = torch.tensor([i % 11 for i in range(T)], dtype=torch.int32)
    zero = torch.full((7,), 5, dtype=torch.int32, device="cuda")
    x, h = residual_embed(toks.cuda(), emb.cuda(), 3.25, w.cuda(), Norm(width, 1e-3), zero)
    want = 3.25 * emb[toks.long()].double()
    tol = 2e-6 if dtype == F32 else 5e-3
    assert rel_err(x, want) < 1e-6 and (zero == 0).all()
    assert rel_err(h[:, :width], O.rms_norm(want[:, :width], w[:width].double(), 1e-3)) < tol and (h[:, width:] == 0).all()
    a = pad(rnd(T, width, seed=5, dtype=dtype))
    pos = torch.tensor([[(3 * t + j) % (2 * T) if (t + j) % 4 else -1 for j in range(2)] for t in range(T)], dtype=torch.int32)
    for y in (pad(rnd(2 * T, width, seed=6, dtype=dtype)), pad(rnd(3, 2 * T, width, seed=7)), None):
        x2 = x.clone()
        e = None if y is None else ExpertRows(y.cuda(), pos.cuda())
        h = residual_add(x2, a.cuda(), ab.cuda(), e, w2.cuda(), Norm(width, 1e-5), dtype)
        s = want + a.double() + ab.double()
        if y is not None:
            ys = y.double() if y.dim() == 2 else y.double().sum(0)
            for t in range(T):
                for p in pos[t].tolist():
                    if p >= 0:
                        s[t] += ys[p]
        assert rel_err(x2, s) < 1e-6
        assert rel_err(h[:, :width], O.rms_norm(s[:, :width], w2[:width].double(), 1e-5)) < tol


# -------------------------------------------------------------------- experts
MOE = [  # tokens, experts, top, width, ff, limit
    (1, 4, 1, 128, 128, 1.0), (7, 5, 2, 256, 128, 0.7), (65, 20, 3, 512, 256, 1.5), (300, 3, 3, 256, 384, 0.4),
    (700, 2, 1, 256, 128, 1.0), (33, 130, 8, 128, 128, 2.0), (19, 64, 5, 384, 128, 1.0), (1025, 100, 4, 128, 128, 1.0)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("T,E,top,W,ff,limit", MOE)
def test_experts(T, E, top, W, ff, limit, dtype):
    """Routing, the sorted order and both grouped products: every choice's row is its
    expert's output for the token's weighted input."""
    from kgs.ops import moe as M
    from kgs.ops.activation import Gate

    W256 = (W + 255) // 256 * 256
    pad = lambda t, n, d: torch.nn.functional.pad(t, (0, W256 - W) if d == 1 else (0, 0, 0, W256 - W))  # noqa: E731
    h = pad(rnd(T, W, seed=T, dtype=dtype), W256, 1)
    ep = next((s for s in (16, 32, 64) if s >= E), (E + 15) // 16 * 16)
    router = torch.zeros(ep, W256, dtype=dtype)
    router[:E] = pad(rnd(E, W, seed=2, scale=W ** -0.5, dtype=BF).to(dtype), W256, 1)
    gu = pad(rnd(E * 2 * ff, W, seed=3, scale=2 * W ** -0.5, dtype=BF).to(dtype), W256, 1).reshape(E, 2 * ff, W256)
    dn = pad(rnd(E, W, ff, seed=4, scale=ff ** -0.5, dtype=BF).to(dtype), W256, 0).contiguous()
    slots = torch.arange(T, dtype=torch.int32)
    if T > 2:
        slots[T // 2] = -1  # a padding row
    counts = torch.zeros(E, dtype=torch.int32, device="cuda")
    c = M.route(h.cuda(), router.cuda(), counts, top, slots.cuda())
    hd = h.double()
    idx, wt = O.route(hd, router[:E].double(), top)
    real = slots >= 0
    z = torch.sigmoid(hd @ router[:E].double().T)
    ids = c.ids.cpu().long()
    assert (ids[~real] == -1).all()
    # the chosen scores (near ties may swap experts)
    assert torch.allclose(z[real].gather(1, ids[real]), wt[real], atol=1e-5)
    assert torch.allclose(c.weight.cpu()[real].double(), wt[real], atol=1e-5)
    assert all(len(set(r)) == top for r in ids[real].tolist())
    assert counts.cpu().tolist() == [int((ids == e).sum()) for e in range(E)]
    p = M.plan(c, M.tile_rows(T, top, E, dtype))
    n = int(real.sum()) * top
    pos = p.pos.cpu()
    assert sorted(pos[real].reshape(-1).tolist()) == list(range(n)) and (pos[~real] == -1).all()
    a = M.gate_up(h.cuda(), gu.cuda(), p, Gate("clamped", limit))
    y = M.down(a, dn.cuda(), p)
    y = (y if y.dim() == 2 else y.sum(0)).cpu()
    check = range(T) if T < 100 else np.random.default_rng(0).integers(0, T, 60).tolist()
    got, want = [], []
    for t in check:
        if not real[t]:
            continue
        for j in range(top):
            e = int(ids[t, j])
            got.append(y[pos[t, j]])
            want.append(O.expert(z[t, e] * hd[t], gu[e, :ff].double(), gu[e, ff:].double(), dn[e].double(), limit))
    got, want = torch.stack(got), torch.stack(want)
    assert rel_err(got, want) < (1e-5 if dtype == F32 else 2e-2)
    if dtype == BF:  # the split form and the whole one agree
        full = M._grouped(a, dn.cuda(), torch.empty((a.shape[0], W256), dtype=BF, device="cuda"), p, a.shape[0], 1, None)
        assert rel_err(full[:n].cpu(), y[:n].double()) < 1e-2


def test_router_reads_32_bit_sums():
    """Two experts whose logits differ in the last bits of an fp32 sum of exact
    products: the larger wins, at every position of a tile."""
    from kgs.ops import moe as M

    W, T, E = 1024, 40, 7
    h = torch.ones(T, W, dtype=BF)
    w = torch.zeros(16, W, dtype=BF)
    w[:E] = 0.5
    w[4, 17] = 0.50390625     # one bf16 step above: 2^-8 of a sum of 512
    counts = torch.zeros(E, dtype=torch.int32, device="cuda")
    c = M.route(h.cuda(), w.cuda(), counts, 2)
    assert (c.ids[:, 0] == 4).all() and (c.ids[:, 1] == 0).all()  # ties: the lower number


# ------------------------------------------------------------------ attention
SHAPES = [  # heads, kv_heads, dim, vdim
    (9, 3, 56, 40), (1, 1, 16, 16), (5, 1, 80, 128), (8, 8, 64, 64), (12, 3, 128, 64), (20, 4, 100, 50), (32, 8, 128, 128),
    (16, 4, 128, 128), (28, 7, 40, 120), (18, 18, 32, 64), (40, 5, 64, 100), (64, 16, 128, 128), (4, 2, 160, 32),
    (66, 6, 20, 40)]


class Case:
    """Sequences with scattered pages, every token's k and v in them."""

    def __init__(self, shape, lens, dtype, far=50.0, rows=16, seed=0, talk=None, sharp=()):
        from kgs.ops.decode import PAGE
        from kgs.ops.talking import TalkingWeights, heads_of, write_kv

        H, G, D, V = shape
        self.h = h = heads_of(H, G, D, V, dtype)
        self.dtype, self.lens = dtype, lens
        T = sum(lens)
        q, k, v = (rnd(T, n, d, seed=seed + i, dtype=dtype) for i, (n, d) in enumerate(((H, D), (G, D), (G, V))))
        for t, j, f in sharp:  # row t's queries find row j's key
            k[j] = q[t].reshape(G, H // G, D)[:, 0] * f
        b = [rnd(n * d, seed=seed + 5 + i, scale=0.5, dtype=BF).float() for i, (n, d) in enumerate(((H, D), (G, D), (G, V)))]
        self.scale = D ** -0.5
        self.talk = (torch.eye(H) + rnd(H, H, seed=seed + 9, scale=0.5 * H ** -0.5)).to(BF) if talk is None else talk
        self.temp = (1 + rnd(H, seed=seed + 10, scale=0.2)).to(BF)
        self.rel, self.far = rnd(rows, H, seed=seed + 11, dtype=BF), far
        pad = lambda t, p: torch.nn.functional.pad(t, (0, p - t.shape[-1]))  # noqa: E731
        parts = [pad(q, h.dkp).reshape(T, -1), pad(k, h.dkp).reshape(T, -1), pad(v, h.dvp).reshape(T, -1)]
        z = torch.cat([parts[0], torch.full((T, 8), 7.0, dtype=dtype), *parts[1:]], 1)
        self.ok = parts[0].shape[1] + 8
        self.ov = self.ok + parts[1].shape[1]
        bias = torch.cat([pad(x.reshape(n, -1), p).reshape(-1) for x, n, p in zip(b, (H, G, G), (h.dkp, h.dkp, h.dvp))])
        rng = np.random.default_rng(seed)
        per = [-(-n // PAGE) for n in lens]
        pages = 1 + rng.permutation(sum(per))
        self.W = max(per) + 1
        self.bt = np.zeros((len(lens), self.W), np.int32)
        slots, at = [], 0
        for i, (n, c) in enumerate(zip(lens, per)):
            self.bt[i, :c] = pages[at:at + c]
            slots += [self.bt[i, t // PAGE] * PAGE + t % PAGE for t in range(n)]
            at += c
        self.pages = torch.zeros((sum(per) + 1, G, PAGE * (h.dkp + h.dvp)), dtype=dtype, device="cuda")
        self.z = z.cuda()
        write_kv(self.z, bias.cuda(), self.pages, torch.tensor(slots, dtype=torch.int32).cuda(), h, self.ok, self.ov)
        self.w = TalkingWeights(h, self.talk, self.temp, self.rel, self.scale, far, "cuda")
        rd = lambda t: t.to(dtype).double()  # noqa: E731
        self.q, self.k, self.v = (rd(t.float() + x.reshape(1, t.shape[1], -1)) for t, x in zip((q, k, v), b))

    def oracle(self, i):
        """``[n, H, V]`` of sequence i."""
        r0 = sum(self.lens[:i])
        q, k, v = (t[r0:r0 + self.lens[i]] for t in (self.q, self.k, self.v))
        s = O.scores(q, k, self.scale, self.temp.double()) + O.distance_bias(self.rel.double(), self.far, len(q))
        p = O.softmax_plus_one(O.talk(s, self.talk.double()))
        H, G = q.shape[1], k.shape[1]
        return torch.stack([p[..., x] @ v[:, x // (H // G)] for x in range(H)], 1)

    def out(self):
        return torch.full((sum(self.lens), self.h.heads * self.h.dvp), float("nan"), dtype=self.dtype, device="cuda")

    def view(self, o):
        return o.reshape(len(o), self.h.heads, self.h.dvp)

    def rows(self, sel, nsplit):
        """``sel``: (sequence, position) pairs."""
        from kgs.ops.talking import QueryRows, attention_rows

        base = np.cumsum([0] + self.lens)
        i32 = lambda a: torch.tensor(a, dtype=torch.int32).cuda()  # noqa: E731
        r = QueryRows(len(sel), i32(self.bt), i32([s for s, _ in sel]), i32([p for _, p in sel]),
                      i32([base[s] + p for s, p in sel]), nsplit)
        return self.view(attention_rows(self.z, self.pages, self.w, r, self.out()))

    def tiles(self, portions, split=False):
        """``portions``: (sequence, first position, tokens)."""
        from kgs.ops.talking import QueryTiles, attention_tiles, tile_items

        base = np.cumsum([0] + self.lens)
        items, merges = tile_items([(base[s] + p, s, p, n) for s, p, n in portions], self.h.tile)
        assert split == bool(len(merges))
        i32 = lambda a: torch.tensor(a, dtype=torch.int32).cuda()  # noqa: E731
        t = QueryTiles(i32(items), i32(self.bt), i32(merges) if split else None, int(merges[:, 3].sum()))
        return self.view(attention_tiles(self.z, self.pages, self.w, t, self.out()))

    def check(self, got, sel, what):
        base, tol = np.cumsum([0] + self.lens), 2e-5 if self.dtype == F32 else 2e-2
        want = {s: self.oracle(s) for s in {s for s, _ in sel}}
        V = self.v.shape[2]
        for s, p in sel:
            g, w = got[base[s] + p].detach().cpu().double(), want[s][p]
            assert (g[:, V:] == 0).all(), (what, s, p)
            err = float((g[:, :V] - w).abs().max()) / float(want[s].abs().max())
            assert err < tol, f"{what}: sequence {s} position {p} off by {err:.1e}"


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("shape", SHAPES, ids=str)
def test_attention(shape, dtype):
    """Single tokens at page borders and splits, whole prompts and portions at any
    position, against the oracle; rows that were not asked for stay as they were."""
    c = Case(shape, [1, 70, 131, 33], dtype)
    sel = [(0, 0), (1, 0), (1, 31), (1, 32), (1, 69), (2, 0), (2, 63), (2, 64), (2, 65), (2, 130), (3, 32)]
    for nsplit in (1, 2, 5):
        got = c.rows(sel, nsplit)
        c.check(got, sel, f"rows / {nsplit}")
        assert int(torch.isnan(got[:, 0, 0]).sum()) == sum(c.lens) - len(sel)
    if c.h.tiled:
        portions = [(0, 0, 1), (1, 0, 70), (2, 0, 40), (2, 40, 16), (2, 56, 17), (2, 73, 58), (3, 5, 28)]
        got = c.tiles(portions)
        c.check(got, [(s, p + j) for s, p, n in portions for j in range(n)], "tiles")
        assert torch.isnan(got[sum(c.lens[:3]):sum(c.lens[:3]) + 5]).all()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("shape", [(9, 3, 56, 40), (32, 8, 128, 128), (20, 4, 100, 50)], ids=str)
def test_scores_that_stand_out(shape, dtype):
    """Keys that one query finds by far the best -- the first, at page borders, far back,
    the last -- in rising order, so the running maximum moves in late tiles."""
    sharp = [(300, 0, 1.0), (290, 31, 2.0), (250, 32, 3.0), (251, 160, 2.5), (200, 199, 3.0), (299, 64, 2.0), (120, 95, 4.0)]
    c = Case(shape, [301], dtype, sharp=sharp)
    sel = [(0, t) for t, _, _ in sharp]
    c.check(c.rows(sel, 1), sel, "rows")
    c.check(c.rows(sel, 4), sel, "rows / 4")
    if c.h.tiled:
        c.check(c.tiles([(0, 0, 301)]), [(0, p) for p in range(301)], "tiles")
        c.check(c.tiles([(0, 110, 191)]), [(0, p) for p in range(110, 301)], "tiles")


@pytest.mark.parametrize("shape", [(9, 3, 56, 40), (20, 4, 100, 50), (16, 4, 128, 128)], ids=str)
def test_split_tiles(shape):
    """Portions over many pages: blocks split over their pages and merged, beside whole ones."""
    sharp = [(700, 3, 2.0), (690, 512, 2.0), (650, 300, 3.0), (700, 699, 1.0)]
    c = Case(shape, [701, 40], BF, sharp=sharp)
    got = c.tiles([(0, 600, 101), (1, 0, 40)], split=True)
    c.check(got, [(0, p) for p in range(600, 701)] + [(1, p) for p in range(40)], "split tiles")
    assert torch.isnan(got[:600]).all()


@pytest.mark.parametrize("rows,far", [(16, 50.0), (24, 200.0), (2, 7.0), (64, 150.5)])
@pytest.mark.parametrize("dtype", [F32, BF])
def test_every_bucket_edge(rows, far, dtype):
    """One bucket at a time much higher than the others: a distance counted to the
    wrong bucket changes the weights of a whole range of keys."""
    for b in sorted({0, 1, rows // 2 - 1, rows // 2, rows // 2 + 1, rows - 2, rows - 1} & set(range(rows))):
        c = Case((4, 2, 32, 32), [290], dtype, far=far, rows=rows, talk=torch.eye(4, dtype=BF).flip(0), seed=b)
        c.rel = torch.zeros_like(c.rel)
        c.rel[b] = torch.tensor([6.0, -6.0, 4.0, 8.0])
        from kgs.ops.talking import TalkingWeights

        c.w = TalkingWeights(c.h, c.talk, c.temp, c.rel, c.scale, far, "cuda")
        sel = [(0, p) for p in (0, 5, 31, 32, 100, 243, 289)]
        c.check(c.rows(sel, 2), sel, f"rows, bucket {b}")
        if c.h.tiled:
            c.check(c.tiles([(0, 0, 290)]), [(0, p) for p in range(290)], f"tiles, bucket {b}")


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("level", [-30.0, 0.0, 30.0])
def test_the_one_in_the_denominator(level, dtype):
    """All scores far below, about and far above the added term's 0."""
    c = Case((9, 3, 56, 40), [100], dtype)
    c.rel = torch.full_like(c.rel, level)
    c.talk = torch.eye(9, dtype=BF)
    from kgs.ops.talking import TalkingWeights

    c.w = TalkingWeights(c.h, c.talk, c.temp, c.rel, c.scale, c.far, "cuda")
    sel = [(0, p) for p in (0, 1, 40, 99)]
    c.check(c.rows(sel, 1), sel, "rows")
    c.check(c.rows(sel, 3), sel, "rows / 3")
    if c.h.tiled:
        c.check(c.tiles([(0, 0, 100)]), [(0, p) for p in range(100)], "tiles")


def test_mixed_scores_are_32_bit():
    """A large score that two heads share and the mixture subtracts again: what is left
    is right only if the mixture keeps the scores' low bits."""
    H = 8
    talk = torch.eye(H)
    talk[0, 1] = -1.0
    c = Case((H, 2, 64, 64), [64], BF, talk=talk.to(BF))
    # heads 0 and 1 share a key head: equal queries but for a small part
    q = c.z[:, :H * 64].reshape(64, H, 64)
    q[:, 1] = q[:, 0] * 16
    q[:, 0] = q[:, 1]
    q[:, 0, 5] += 0.5
    c.q = c.z[:, :H * 64].reshape(64, H, 64).cpu().double()
    c.temp = torch.ones(H, dtype=BF)
    c.rel = torch.zeros_like(c.rel)
    from kgs.ops.talking import TalkingWeights

    c.w = TalkingWeights(c.h, c.talk, c.temp, c.rel, c.scale, c.far, "cuda")
    want = c.oracle(0)[:, 0]
    for got in (c.rows([(0, p) for p in range(64)], 1), c.tiles([(0, 0, 64)])):
        err = (got[:, 0].cpu().double() - want).abs().max() / want.abs().max()
        assert err < 1e-2, float(err)


@pytest.mark.parametrize("dtype", [F32, BF])
def test_write_kv_forms(dtype):
    """Aligned runs of 8 tokens, broken runs, dropped rows: the same pages as one by one."""
    from kgs.ops.talking import heads_of, write_kv

    h = heads_of(4, 2, 64, 64, dtype)
    n = 4 * 64 + 2 * 128
    b = rnd(n, seed=1).cuda()
    slots = [*range(32, 56), *range(57, 64), 70, -1, 71, 9, 8, *range(96, 104), -1, 90]
    z = rnd(len(slots), n, seed=2, dtype=dtype).cuda()
    one, all_ = (torch.zeros(4, 2, 32 * 128, dtype=dtype, device="cuda") for _ in range(2))
    z2 = z.clone()
    write_kv(z2, b, all_, torch.tensor(slots, dtype=torch.int32).cuda(), h, 256, 384)
    for i, s in enumerate(slots):
        write_kv(z[i:i + 1], b, one, torch.tensor([s], dtype=torch.int32).cuda(), h, 256, 384)
    assert torch.equal(one, all_) and torch.equal(z, z2)
    k = (z2[3, 256:320].float() + 0)  # k and v of z stay; only q has its bias
    # token slot 35 of page 1, key head 0: dim d at its place in fragment order
    for d in (0, 7, 8, 31, 32, 63):
        t = 35 % 32
        at = (((t & 1) * 2 + d // 32) * 64 + (d // 8) % 4 * 16 + (t >> 1)) * 8 + d % 8
        assert all_[1, 0, at] == (k[d] + b[256 + d]).to(dtype)
        at = 32 * 64 + (d // 16 * 64 + t // 8 * 16 + d % 16) * 8 + t % 8
        assert all_[1, 0, at] == (z2[3, 384 + d].float() + b[384 + d]).to(dtype)


def test_shapes_the_kernels_refuse():
    from kgs.ops._lib import KernelError
    from kgs.ops.talking import attention_tiles

    c = Case((18, 18, 32, 64), [40], BF)
    with pytest.raises(ValueError, match="no tiled kernel"):
        attention_tiles(c.z, c.pages, c.w, None, c.out())
    from kgs.ops import moe as M

    with pytest.raises((KernelError, ValueError)):
        M.route(torch.zeros(2, 100, dtype=BF, device="cuda"), torch.zeros(16, 100, dtype=BF, device="cuda"),
                torch.zeros(4, dtype=torch.int32, device="cuda"), 2)
