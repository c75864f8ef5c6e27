"""Vumalix's kernels one by one against plain references: the post-normed residual with its
convolution and state, normed powers, head norms and the query temperature in the cache
write, differential attention (rows, tiles, plain), rotated keys, windows and element gates
of latent attention in both forms -- with inputs that stand out where a fault would hide."""
import math
import os
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

from oracles import vumalix as O  # noqa: E402

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
def ragged(n, pos0, slots):
    from kgs.ops.delta import RaggedSeqs

    n = np.asarray(n)
    return RaggedSeqs(i32(np.repeat(np.arange(len(n)), n)), i32(np.cumsum(n) - n), i32(n), i32(pos0), i32(slots))


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width,wp,taps", [(140, 256, 1), (140, 256, 2), (140, 256, 3), (512, 512, 4), (520, 768, 6), (4096, 4096, 3),
                                           (5000, 5120, 4), (8200, 8448, 2), (64, 256, 40)])
def test_residual_steps_over_ragged_portions(dtype, width, wp, taps):
    """Three requests in portions from one token on, in slots that held rubbish: embedding and
    convolution, a sublayer's normed output added before another convolution with a state of
    its own, a plain step, the final norm."""
    from kgs.ops.postnorm import Conv, ConvState, PostNorm, Sublayer

    eps, vocab = 1e-2, 11
    pad = lambda t: torch.nn.functional.pad(t, (0, wp - width))  # noqa: E731
    emb = pad(rnd(vocab, width, seed=1, dtype=dtype))
    convs = [rnd(width, taps, seed=2 + i, scale=0.5) for i in range(2)]
    dev = [Conv(c.cuda(), wp) for c in convs]
    states = [ConvState(taps, wp, 5, "cuda") for _ in range(2)]
    for s in states:
        s.rows.fill_(float("nan"))  # position 0 must not read it
    save = [s if taps > 1 else None for s in states]
    lens, slots = [45, 9, 30], [3, 1, 4]
    toks = [np.random.default_rng(i).integers(0, vocab, n) for i, n in enumerate(lens)]
    ys = [[rnd(n, width, seed=10 * i + j, scale=3.0, dtype=dtype) for j in range(3)] for i, n in enumerate(lens)]
    x0 = [emb[torch.as_tensor(t), :width].double() for t in toks]
    x1 = [x + 0.7 * O.rms(y[0].double(), eps) for x, y in zip(x0, ys)]
    x2 = [x - 1.3 * O.rms(y[1].double(), eps) for x, y in zip(x1, ys)]
    x3 = [x + 0.4 * O.rms(y[2].double(), eps) for x, y in zip(x2, ys)]
    want = [[x + O.causal_conv(x, convs[0].double()) for x in x0], x1, [x + O.causal_conv(x, convs[1].double()) for x in x2],
            [1.7 * O.rms(x, eps) for x in x3], x3]
    got = [[[] for _ in lens] for _ in want]
    at = [0, 0, 0]
    tol = 3e-6 if dtype == F32 else 5e-3
    for step in ([20, 1, 0], [1, 1, 2], [2, 2, 1], [0, 1, 17], [1, 0, 1], [21, 4, 9]):
        seq = [i for i, n in enumerate(step) if n]
        cut = lambda src: torch.cat([src(i)[at[i]:at[i] + step[i]] for i in seq])  # noqa: E731
        sq = ragged([step[i] for i in seq], [at[i] for i in seq], [slots[i] for i in seq])
        res = PostNorm(i32(cut(lambda i: torch.as_tensor(toks[i]))), sq, width, wp, eps, dtype)
        sub = lambda j, g: Sublayer(pad(cut(lambda i: ys[i][j])).cuda(), g)  # noqa: E731
        outs = [res.start(emb.cuda(), dev[0], states[0]), res.add(sub(0, 0.7), save=save[0]),
                res.add(sub(1, -1.3), dev[1], states[1]), res.close(sub(2, 0.4), 1.7, save=save[1])]
        outs.append(res.x)
        for k, o in enumerate(outs):
            assert (o[:, width:] == 0).all()
            r = 0
            for i in seq:
                got[k][i].append(o[r:r + step[i], :width].float().cpu())
                r += step[i]
        for i in seq:
            at[i] += step[i]
    assert at == lens
    for k in range(len(want)):
        for i in range(3):
            err = rel_err(torch.cat(got[k][i]), want[k][i])
            assert err < (3e-6 if k == 4 else tol), (k, i, err)


def test_residual_of_a_long_batch():
    """More rows than compute units, portions of every length; the state is one of the rows."""
    from kgs.ops.postnorm import Conv, ConvState, PostNorm, Sublayer

    width, taps, eps = 256, 3, 1e-5
    n = np.random.default_rng(0).integers(1, 60, 100)
    T = int(n.sum())
    emb, conv = rnd(50, width, seed=1, dtype=BF), rnd(width, taps, seed=2)
    toks, y = np.random.default_rng(1).integers(0, 50, T), rnd(T, width, seed=3, dtype=BF)
    state = ConvState(taps, width, 101, "cuda")
    res = PostNorm(i32(toks), ragged(n, np.zeros(100), 1 + np.arange(100)), width, width, eps, BF)
    c = Conv(conv.cuda(), width)
    h0 = res.start(emb.cuda(), c, state)
    h1 = res.add(Sublayer(y.cuda(), 1.5), c, state, save=ConvState(taps, width, 101, "cuda"))
    rows, at = emb[torch.as_tensor(toks)].double(), 0
    x1 = rows + 1.5 * O.rms(y.double(), eps)
    for m in n:
        for h, x in ((h0, rows), (h1, x1)):
            x = x[at:at + m]
            assert rel_err(h[at:at + m], x + O.causal_conv(x, conv.double())) < 5e-3
        at += m


# --------------------------------------------------------------- normed powers
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("n,np_", [(72, 128), (200, 256), (257, 320), (512, 512), (4100, 4224), (14336, 14336), (20000, 20096)])
def test_normed_powers(dtype, n, np_):
    """Rows of different sizes, one far beyond the others (a norm over the batch would show) and
    one near zero, where eps decides."""
    from kgs.ops.activation import poly_norm

    z = rnd(5, n, seed=n, dtype=dtype) * torch.tensor([1.0, 30.0, 0.01, 1.0, 3.0], dtype=dtype)[:, None]
    wide = torch.nn.functional.pad(z, (0, np_ - n + 64))
    act = torch.tensor([0.7, -0.5, 0.3, 0.25])
    out = poly_norm(wide.cuda()[:, :np_], act.cuda(), n, 1e-3)
    assert out.shape == (5, np_) and torch.isfinite(out.float()).all()
    for r in range(5):
        assert rel_err(out[r, :n], O.poly_norm(z[r].double(), act.double(), 1e-3)) < (3e-6 if dtype == F32 else 5e-3)


# ------------------------------------------------------ differential attention
class Case:
    """Sequences with scattered pages; q, k and v as a projection leaves them, keys and values
    written by the product's own write, which norms and scales."""

    def __init__(self, shape, lens, dtype, seed=0, sharp=(), eps=1e-3, temp=(0.7, 13), lam=0.45, diff=0.3):
        from kgs.ops.paged import Differential, paged_heads
        from kgs.ops.talking import HeadNorm, HeadPages, Temperature, write_kv

        H, G, d, dv = shape
        self.lens, self.dtype, self.dv = lens, dtype, dv
        self.h = h = paged_heads(H, G, d, dv, dtype, maps=2)
        seg = h.dkp // 2
        T = sum(lens)
        self.scale = 1.1 * d ** -0.5
        self.diff = Differential(lam, 1 - diff, dv, eps)
        q, k, v = rnd(T, H, 2, d, seed=seed, scale=2), rnd(T, G, 2, d, seed=seed + 1, scale=0.5), rnd(T, G, dv, seed=seed + 2)
        wq, wk = 1 + rnd(d, seed=seed + 3, scale=0.3), 1 + rnd(d, seed=seed + 4, scale=0.3)
        for i, j, m in sharp:  # map m of query i of the first sequence finds key j by far the best
            for x in range(H):
                q[i, x, m] = k[j, x // (H // G), m] * wk / wq
        q, k, v = (t.to(dtype) for t in (q, k, v))
        pads = lambda t, s: torch.nn.functional.pad(t, (0, s - t.shape[-1]))  # noqa: E731
        offs = [0, -(-H * h.dkp // 64) * 64]
        offs.append(offs[1] + -(-G * h.dkp // 64) * 64)
        z = torch.zeros(T, offs[2] + G * h.dvp + 64, dtype=dtype)
        z[:, :H * h.dkp] = pads(q, seg).reshape(T, -1)
        z[:, offs[1]:offs[1] + G * h.dkp] = pads(k, seg).reshape(T, -1)
        z[:, offs[2]:offs[2] + G * h.dvp] = pads(v, h.dvp).reshape(T, -1)
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
        write_kv(self.z, None, self.pages, i32(slots), h, offs[1], offs[2], pos=i32(pos),
                 norm=HeadNorm(pads(wq, seg).cuda(), pads(wk, seg).cuda(), d, eps), temperature=Temperature(*temp))
        base = np.cumsum([0] + lens)
        self.want, self.queries = [], []
        for s in range(len(lens)):
            sl = slice(base[s], base[s + 1])
            n = lens[s]
            t = O.temperature(n, {"coef": temp[0], "every": temp[1]}, torch.float64)
            qs = O.rms(q[sl].double(), eps) * wq.double() * t[:, None, None, None]
            ks, vs = O.rms(k[sl].double(), eps) * wk.double(), v[sl].double()
            self.queries.append(qs)
            mask, out = O.window_mask(n, n), []
            for x in range(H):
                g = x // (H // G)
                a1, a2 = (O.weighted(qs[:, x, m] @ ks[:, g, m].T * self.scale, mask, vs[:, g]) for m in range(2))
                out.append(O.rms(a1 - lam * a2, eps) * (1 - diff))
            self.want.append(torch.stack(out, 1))

    def out(self):
        return torch.full((sum(self.lens), self.h.heads * self.h.dvp), float("nan"), dtype=self.dtype, device="cuda")

    def rows(self, sel, nsplit):
        from kgs.ops.paged import paged_rows
        from kgs.ops.talking import QueryRows

        base = np.cumsum([0] + self.lens)
        r = QueryRows(len(sel), i32(self.bt), i32([s for s, _ in sel]), i32([p for _, p in sel]),
                      i32([base[s] + p for s, p in sel]), nsplit)
        return paged_rows(self.z, self.pages, self.h, self.scale, 0, r, self.out(), self.diff)

    def tiles(self, portions):
        from kgs.ops.paged import Portions, paged_tiles, portion_items, tile_queries

        base = np.cumsum([0] + self.lens)
        items = portion_items([(base[s] + p, s, p, n) for s, p, n in portions], tile_queries(self.h), 0)
        return paged_tiles(self.z, self.pages, self.h, self.scale, 0, Portions(i32(items), i32(self.bt)), self.out(), self.diff)

    def check(self, got, sel, what):
        base, tol = np.cumsum([0] + self.lens), 3e-5 if self.dtype == F32 else 4e-2
        got = got.cpu().double().reshape(len(got), self.h.heads, self.h.dvp)
        assert int(torch.isfinite(got[:, 0, 0]).sum()) == len(set(sel)), what  # and no other row
        for s, p in sel:
            g, w = got[base[s] + p], self.want[s][p]
            assert (g[:, self.dv:] == 0).all(), (what, s, p)
            err = float((g[:, :self.dv] - w).abs().max()) / float(self.want[s].abs().max())
            assert err < tol, f"{what}: sequence {s} position {p} off by {err:.1e}"


# heads, kv heads, dim of a map, vdim: groups of 1, 2, 4, 9, 16 and 64 heads; sizes the MFMA kernels pad or leave
SHAPES = [(4, 2, 24, 40), (5, 5, 64, 128), (16, 4, 128, 128), (18, 2, 100, 64), (16, 1, 64, 64), (64, 1, 64, 100),
          (6, 3, 160, 80), (2, 1, 16, 300), (3, 3, 40, 20)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("shape", SHAPES, ids=str)
def test_differential_attention(shape, dtype):
    """Single tokens at page borders and splits, whole prompts and portions at any position;
    rows that were not asked for stay as they were."""
    from kgs.ops.paged import tile_queries

    c = Case(shape, [1, 70, 131, 33], dtype)
    sel = [(0, 0), (1, 0), (1, 1), (1, 31), (1, 32), (1, 69), (2, 63), (2, 64), (2, 95), (2, 96), (2, 130), (3, 32)]
    for nsplit in (1, 2, 5):
        c.check(c.rows(sel, nsplit), sel, f"rows / {nsplit}")
    if tile_queries(c.h):
        portions = [(0, 0, 1), (1, 0, 70), (2, 0, 40), (2, 40, 16), (2, 56, 17), (2, 73, 58), (3, 5, 28)]
        c.check(c.tiles(portions), [(s, p + j) for s, p, n in portions for j in range(n)], "tiles")
    else:
        assert dtype == F32 or shape in SHAPES[6:]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("shape", [(9, 3, 56, 40), (16, 4, 64, 128), (4, 4, 128, 128)], ids=str)
def test_scores_that_stand_out_in_one_map(shape, dtype):
    """Keys that one map of a query finds by far the best -- the first, at page borders, far
    back, the query's own: seen by that map, not by the other one."""
    from kgs.ops.paged import tile_queries

    sharp = [(299, 0, 0), (290, 256, 1), (288, 255, 0), (198, 99, 1), (99, 31, 0), (120, 120, 1),
             (255, 32, 0)]
    c = Case(shape, [301], dtype, sharp=sharp, temp=(1.5, 20))
    sel = [(0, t) for t, *_ in sharp]
    c.check(c.rows(sel, 1), sel, "rows")
    c.check(c.rows(sel, 4), sel, "rows / 4")
    if tile_queries(c.h):
        c.check(c.tiles([(0, 0, 301)]), [(0, p) for p in range(301)], "tiles")
        c.check(c.tiles([(0, 110, 191)]), [(0, p) for p in range(110, 301)], "tiles")


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("d", [16, 64, 72, 128, 200])
def test_head_norm_and_temperature(d, dtype):
    """Queries in place and keys in the cache, with lanes of a norm that share a wave or not."""
    c = Case((6, 2, d, 32), [75], dtype, temp=(0.9, 10))
    got = c.z[:, :6 * c.h.dkp].float().cpu().reshape(75, 6, 2, -1)
    for p in (0, 8, 9, 10, 18, 19, 74):  # the temperature's steps are at 9, 19, ..
        assert rel_err(got[p, ..., :d], c.queries[0][p]) < (3e-6 if dtype == F32 else 5e-3), p
    assert (got[..., d:] == 0).all()
    f = 1 + 0.9 * math.log(8)
    assert abs(f - float(O.temperature(75, {"coef": 0.9, "every": 10}, torch.float64)[74])) < 1e-12


def test_temperature_far_out():
    from kgs.ops.paged import paged_heads
    from kgs.ops.talking import HeadNorm, HeadPages, Temperature, write_kv

    h = paged_heads(1, 1, 64, 64, F32, maps=2)
    pages = HeadPages({0: h}, 2, F32, "cuda").pages[0]
    z = torch.ones(4, 320, device="cuda")
    one = torch.ones(64, device="cuda")
    pos = [0, 8190, 8191, 200000]
    write_kv(z, None, pages, i32([-1] * 4), h, 128, 256, pos=i32(pos), norm=HeadNorm(one, one, 64, 0.0),
             temperature=Temperature(0.1, 8192))
    want = torch.tensor([1 + 0.1 * math.log((p + 1) // 8192 + 1) for p in pos])
    assert torch.allclose(z[:, 0].cpu(), want, rtol=1e-6) and torch.allclose(z[:, 127].cpu(), want, rtol=1e-6)
    assert (z[:, 128:] == 1).all() and (pages == 0).all()


# ------------------------------------------------------------ latent attention
def turned(x, base):
    """Neighbouring pairs (the layout behind the projections), rows at their positions."""
    if x.dim() == 2:
        return turned(x[:, None], base)[:, 0]
    half = torch.cat([x[..., 0::2], x[..., 1::2]], -1)
    t = O.rotate_half(half, base)
    h = x.shape[-1] // 2
    return torch.stack([t[..., :h], t[..., h:]], -1).flatten(-2)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("nq,nc,rot", [(96, 72, 16), (20, 64, 2), (130, 250, 64), (40, 512, 20), (64, 96, 100)])
def test_latent_norms_and_the_rotated_key(nq, nc, rot, dtype):
    from kgs.ops.latent import latent_norm, padded_latent, padded_rot
    from kgs.ops.talking import Rotary

    T, eps, base = 90, 1e-4, 50.0
    rp, hr = padded_latent(nc), padded_rot(rot)
    oc = 64 + (nq + 63) // 64 * 64
    okr = oc + (nc + 63) // 64 * 64
    z = rnd(T, okr + (rot + 63) // 64 * 64, dtype=dtype)
    z[:, okr + rot:] = 0  # as the padded projection leaves it
    wq, wc = 1 + 0.1 * rnd(nq, seed=1), 1 + 0.1 * rnd(nc, seed=2)
    pages = torch.full((4, 32, rp + hr), 7.0, dtype=dtype, device="cuda")
    slots = np.random.default_rng(0).permutation(128)[:T]
    slots[5] = -1
    pos = torch.arange(T, dtype=torch.int32, device="cuda")
    cq = latent_norm(z.cuda(), 64, wq.cuda(), 192, oc, wc.cuda(), pages, i32(slots), eps, rp, okr, Rotary(rot, base, T, "cuda"), pos)
    tol = 3e-6 if dtype == F32 else 8e-3
    assert rel_err(cq[:, :nq], O.rms(z[:, 64:64 + nq].double(), eps) * wq.double()) < tol
    c = O.rms(z[:, oc:oc + nc].double(), eps) * wc.double()
    kr = turned(z[:, okr:okr + rot].double(), base)
    flat, keep = pages.view(128, -1).float().cpu(), torch.ones(128, dtype=torch.bool)
    for t, s in enumerate(slots.tolist()):
        if s < 0:
            continue
        assert rel_err(flat[s, :nc], c[t]) < tol and rel_err(flat[s, rp:rp + rot], kr[t]) < tol, t
        assert (flat[s, nc:rp] == 0).all() and (flat[s, rp + rot:] == 0).all()
        keep[s] = False
    assert (flat[keep] == 7).all()  # nothing else is touched


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("nt", [1, 17, 40, 130])
def test_head_proj_gates_elements_and_turns_queries(nt, dtype):
    from kgs.ops.latent import head_proj
    from kgs.ops.talking import Rotary

    H, N, K, rot, hr, R, base = 3, 96, 64, 20, 32, 150, 30.0
    w = rnd(H, N, K, seed=1, dtype=dtype)
    rows = torch.from_numpy(np.random.default_rng(nt).permutation(R)[:nt].astype(np.int32))
    q = rnd(R, H, K + hr, seed=2, dtype=dtype)
    q[:, :, K + rot:] = 0
    pos = torch.arange(nt, dtype=torch.int32) * 3 % nt
    out = torch.full((nt, H * (N + hr)), 9.0, dtype=dtype, device="cuda")
    head_proj(q.reshape(R, -1).cuda(), w.cuda(), nt, out, rows_in=rows.cuda(), hr=hr, rotary=Rotary(rot, base, nt, "cuda"),
              pos=pos.cuda())
    got, tol = out.float().cpu().reshape(nt, H, N + hr), 3e-6 if dtype == F32 else 8e-3
    picked = q[rows.long()].double()
    assert rel_err(got[..., :N], (picked[:, :, None, :K] * w.double()).sum(-1)) < tol
    at = torch.zeros(nt, H, rot, dtype=torch.float64)  # row p of the turned table is position p
    for i, p in enumerate(pos.tolist()):
        spread = torch.zeros(p + 1, H, rot, dtype=torch.float64)
        spread[p] = picked[i, :, K:K + rot]
        at[i] = turned(spread, base)[p]
    assert rel_err(got[..., N:N + rot], at) < tol and (got[..., N + rot:] == 0).all()
    a, gate = rnd(nt, H * K, seed=3, dtype=dtype), rnd(R, H * N + 8, seed=4, dtype=dtype)
    out = torch.zeros(R, H * N, dtype=dtype, device="cuda")
    head_proj(a.cuda(), w.cuda(), nt, out, rows_out=rows.cuda(), gate=gate.cuda()[:, 8:], each=True)
    want = torch.zeros(R, H, N, dtype=torch.float64)
    want[rows.long()] = (a.double().reshape(nt, H, 1, K) * w.double()).sum(-1) * \
        torch.sigmoid(gate[rows.long(), 8:].double()).reshape(nt, H, N)
    assert rel_err(out, want.reshape(R, -1)) < tol


def run_latent(q, rows, lens, n, H, scale, rp, hr, window, dtype, nsplit=None):
    """``q [sum n, H, rp + hr]``, ``rows [B][len, rp + hr]``: the last n[b] positions of each
    sequence; as the serving plan lays them out."""
    from kgs.ops.latent import LatentRows, latent_attention
    from kgs.serve.hybrid import Geometry
    from kgs.serve.ragged import HostPack

    lens, n = np.asarray(lens), np.asarray(n)
    need = -(-lens // 32)
    ids, bt, at = 1 + np.random.default_rng(0).permutation(need.sum()), np.zeros((len(lens), need.max() + 1), np.int32), 0
    pages = torch.full((need.sum() + 1, 32, rp + hr), 3.0, dtype=dtype)  # what a reused page holds must not matter
    flat = pages.view(-1, rp + hr)
    for b, x in enumerate(rows):
        bt[b, :need[b]] = ids[at:at + need[b]]
        at += need[b]
        p = np.arange(lens[b])
        flat[bt[b][p // 32] * 32 + p % 32] = x
    pos0, row0 = lens - n, np.cumsum(n) - n
    seq = np.repeat(np.arange(len(n)), n)
    pos = pos0[seq] + np.arange(n.sum()) - row0[seq]
    pk = HostPack(torch.device("cuda"))
    (r, shape), _ = Geometry(H, rp, 0, window).lay_out(pk, row0, n, pos0, bt, seq, pos, [None] * 7 + [pk.add(bt), None])
    get = pk.send()
    if nsplit:
        shape["nsplit"] = nsplit
    lr = LatentRows(**{k: None if v is None else get(v) for k, v in r.items()}, **shape)
    o = latent_attention(q.reshape(len(seq), -1).cuda(), pages.cuda(), lr, H, scale, hr, window)
    return o.reshape(len(seq), H, rp)


def ref_latent(q, rows, lens, n, scale, rp, window):
    out, at = [], 0
    for b, x in enumerate(rows):
        x = x.double()
        for i in range(n[b]):
            p = lens[b] - n[b] + i
            vis = x[max(0, p - window + 1) if window else 0:p + 1]
            out.append(torch.softmax(q[at + i].double() @ vis.T * scale, -1) @ vis[:, :rp])
        at += n[b]
    return torch.stack(out)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("window", [0, 1, 31, 32, 33, 100])
@pytest.mark.parametrize("rp,hr,H,nsplit", [(32, 32, 5, None), (64, 64, 17, 2), (96, 0, 3, 1), (128, 32, 40, 3), (192, 64, 2, None),
                                            (256, 32, 9, 2), (384, 64, 16, None), (512, 64, 33, None), (512, 32, 4, 5),
                                            (608, 96, 2, None)])
def test_latent_attention_with_rotated_keys_and_windows(rp, hr, H, nsplit, window, dtype):
    lens, n = [1, 31, 33, 64, 200, 45, 321], [1, 2, 3, 1, 1, 45, 7]
    q = rnd(sum(n), H, rp + hr, scale=1.5, dtype=dtype)
    rows = [rnd(m, rp + hr, seed=i + 1, dtype=dtype) for i, m in enumerate(lens)]
    scale = (rp + hr) ** -0.5
    got = run_latent(q, rows, lens, n, H, scale, rp, hr, window, dtype, nsplit)
    assert rel_err(got, ref_latent(q, rows, lens, n, scale, rp, window)) < (8e-6 if dtype == F32 else 1.5e-2)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("window", [2, 30, 64, 65, 200])
def test_latent_attention_sees_exactly_its_window(window, dtype):
    """One key stands out by 40 in score, by its rotated part alone: at every border it is seen
    if and only if it lies in the query's window."""
    rp, hr, H, L = 64, 32, 2, 330
    d = torch.nn.functional.normalize(rnd(hr, seed=3), dim=0)
    v = torch.nn.functional.normalize(rnd(rp, seed=5), dim=0)
    base = 0.05 * rnd(L, rp + hr, seed=4)
    q = torch.cat([torch.zeros(rp), 10 * d]).expand(9, H, -1).to(dtype).contiguous()
    for key in sorted({k for k in (0, 31, 32, 255, 256, 318, 321, 328, 329, *range(L - 9 - window - 1, L - window + 2)) if 0 <= k < L}):
        c = base.clone()
        c[key] = torch.cat([4 * v, 4 * d])
        got = run_latent(q, [c.to(dtype)], [L], [9], H, 1.0, rp, hr, window, dtype, nsplit=4 if key % 2 else None).cpu().float()
        for i in range(9):
            p = L - 9 + i
            sees = key <= p < key + window
            share = float(got[i, 0] @ v) / 4
            assert (share > 0.95) if sees else (share < 0.1), (key, i, share)


@pytest.mark.parametrize("window", [0, 1, 50, 64, 129, 1000])
@pytest.mark.parametrize("hd,hr,rot", [(64, 0, 0), (64, 32, 16), (128, 32, 32), (128, 64, 64), (64, 64, 40), (128, 0, 0)])
def test_attention_ragged_with_rotated_keys_and_windows(hd, hr, rot, window):
    """The expanded form: portions of any length at any position over the keys their windows
    hold, with a gate per element; rows between them untouched."""
    from kgs.ops.talking import Rotary
    from kgs.ops.transformer import attention_ragged

    H, scale, base = 3, 0.13, 40.0
    lens, n = [300, 129, 64, 77, 513], [300, 129, 1, 70, 130]
    T = sum(n) + 5
    q = rnd(T, H, hd + hr, scale=1.2, dtype=BF)
    q[:, :, hd + rot:] = 0
    gate = rnd(T, H * hd, seed=2, dtype=BF)
    pos = torch.zeros(T, dtype=torch.int32)
    row, at, items, ref, ks, krs = 5, 0, [], torch.full((T, H, hd), 9.0, dtype=torch.float64), [], []
    for s, (L, m) in enumerate(zip(lens, n)):
        first = max(0, L - m - window + 1) if window else 0
        kv, kr = rnd(L, 2 * H * hd, seed=10 + s, dtype=BF), rnd(L, max(rot, 2), seed=20 + s)
        kr = turned(kr.double(), base).to(BF) if rot else kr.to(BF)
        for i in range(0, m, 128):
            items.append([row + i, at, L - m + i - first, min(128, m - i)])
        pos[row:row + m] = L - m + torch.arange(m)
        k, v = (x.reshape(L, H, hd).double() for x in kv.chunk(2, 1))
        qs = torch.zeros(L, H, hd + hr, dtype=torch.float64)
        qs[L - m:] = q[row:row + m].double()
        mask = O.window_mask(L, window or L)[L - m:]
        for x in range(H):
            sc = qs[L - m:, x, :hd] @ k[:, x].T
            if rot:
                sc = sc + turned(qs[:, x, hd:hd + rot], base)[L - m:].to(BF).double() @ kr.double().T
            ref[row:row + m, x] = O.weighted(sc * scale, mask, v[:, x])
        ks.append(kv[first:])
        krs.append(torch.nn.functional.pad(kr[first:, :rot], (0, hr - rot)))
        row, at = row + m, at + L - first
    ref[5:] *= torch.sigmoid(gate[5:].double()).reshape(-1, H, hd)
    out = torch.full((T, H * hd), 9.0, dtype=BF, device="cuda")
    kvd = torch.cat(ks).cuda()
    attention_ragged(q.reshape(T, -1).cuda(), kvd[:, :H * hd], kvd[:, H * hd:], i32(items), H, hd, scale, out, gate=gate.cuda(), each=True,
                     window=window, kr=torch.cat(krs).cuda() if hr else None, rotary=Rotary(rot, base, 600, "cuda") if hr else None,
                     pos=pos.cuda())
    got = out.float().cpu().double().reshape(T, H, hd)
    assert rel_err(got[5:], ref[5:]) < 1.5e-2 and (got[:5] == 9).all()
