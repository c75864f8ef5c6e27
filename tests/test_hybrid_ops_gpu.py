"""The mechanisms of the Ruruzen design on the GPU, each alone against the plain
oracle (float64 on the CPU): hyper-connections, feed-forward and soft cap, latent
norms, head products, latent attention in both forms, the delta rule."""
import os
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

from oracles import ruruzen as O  # noqa: E402

pytestmark = pytest.mark.gpu

DT = {"bf16": torch.bfloat16, "f32": torch.float32}
TOL = {"bf16": 8e-3, "f32": 2e-6}


def rnd(*shape, seed=0, scale=1.0, dtype=torch.float32):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).to(dtype)


def close(got, want, tol):
    got, want = got.detach().cpu().double(), want.double()
    assert got.shape == want.shape, (got.shape, want.shape)
    err = (got - want).abs().max() / want.abs().max().clamp(min=1e-9)
    assert err < tol, f"rel err {err:.2e} > {tol}"


# ------------------------------------------------------------ hyper-connections
@pytest.mark.parametrize("dt", ["bf16", "f32"])
@pytest.mark.parametrize("S,D,T", [(1, 64, 5), (2, 140, 3), (3, 203, 4), (4, 256, 9), (5, 1030, 2), (8, 4096, 3)])
def test_hyper_streams(dt, S, D, T):
    from kgs.ops.hyper import hyper_embed, hyper_step

    dtype, eps, V, ld = DT[dt], 3e-5, 37, (D + 63) // 64 * 64
    emb = rnd(V, ld, seed=1, dtype=dtype)
    w0, w1, w2 = (1 + 0.2 * rnd(D, seed=s) for s in (2, 3, 4))
    win1, win2, wout = (rnd(S, seed=s) for s in (5, 6, 7))
    mix, y = rnd(S, S, seed=8), rnd(T, ld + 4, seed=9, dtype=dtype)
    tok = torch.randint(0, V, (T,), generator=torch.Generator().manual_seed(1)).int()
    c = lambda t: t.cuda()  # noqa: E731
    x, h = hyper_embed(c(tok), c(emb), c(w0), c(win1), c(w1), D, eps, ld=ld)
    ref = O.rms_norm(emb[tok.long(), :D].double(), w0.double(), eps)[:, None].repeat(1, S, 1)
    close(x, ref, 2e-6)
    close(h[:, :D], O.rms_norm(O.hyper_in(ref, win1.double()), w1.double(), eps), TOL[dt])
    assert (h[:, D:] == 0).all()
    # start from streams that differ
    x = torch.randn(T, S, D, device="cuda")
    ref = x.cpu().double()
    h = hyper_step(x, c(y), c(mix), c(wout), c(win2), c(w2), eps, ld=ld)
    ref = O.hyper_out(ref, y[:, :D].double(), mix.double(), wout.double())
    close(x, ref, 2e-6)
    close(h[:, :D], O.rms_norm(O.hyper_in(ref, win2.double()), w2.double(), eps), TOL[dt])
    assert (h[:, D:] == 0).all()
    h2 = hyper_step(x, None, None, None, c(win1), c(w1), eps, dtype=dtype)  # read-out only
    close(x, ref, 2e-6)
    close(h2, O.rms_norm(O.hyper_in(ref, win1.double()), w1.double(), eps), TOL[dt])


@pytest.mark.parametrize("dt", ["bf16", "f32"])
def test_feed_forward_product_and_softcap(dt):
    from kgs.ops.activation import act_mul, softcap

    gu = rnd(7, 2 * 200, scale=3, dtype=DT[dt])
    g, u = gu[:, :200].double(), gu[:, 200:].double()
    close(act_mul(gu.cuda(), "gelu_tanh"), O.gelu_tanh(g) * u, TOL[dt])
    close(act_mul(gu.cuda(), "silu"), O.silu(g) * u, TOL[dt])
    x = rnd(5, 320, scale=20, dtype=DT[dt])
    close(softcap(x.cuda(), 203, 12.5), 12.5 * torch.tanh(x[:, :203].double() / 12.5), 1e-5)
    close(softcap(x.cuda(), 203, 0.0), x[:, :203].double(), 1e-7)


# ------------------------------------------------------------- latent attention
def pages_for(lens, W, seed=0):
    """Scattered pages (page 0 is never used) for sequences of these lengths."""
    need = [-(-n // 32) for n in lens]
    ids = 1 + np.random.default_rng(seed).permutation(sum(need))
    bt, at = np.zeros((len(lens), W), np.int32), 0
    for i, k in enumerate(need):
        bt[i, :k] = ids[at:at + k]
        at += k
    return bt, 1 + sum(need)


def slots_of(bt, b, pos):
    pos = np.asarray(pos)
    return bt[b][pos // 32] * 32 + pos % 32


@pytest.mark.parametrize("dt", ["bf16", "f32"])
@pytest.mark.parametrize("nq,nc", [(96, 72), (20, 0), (130, 250)])
def test_latent_norms_and_cache_write(dt, nq, nc):
    from kgs.ops.latent import latent_norm, padded_latent

    dtype, eps, T = DT[dt], 1e-4, 6
    oq, oc, rp = 64, 64 + (nq + 63) // 64 * 64, padded_latent(nc) if nc else 0
    z = rnd(T, oc + nc + 5, dtype=dtype)
    wq, wc = 1 + 0.1 * rnd(nq, seed=1), 1 + 0.1 * rnd(max(nc, 1), seed=2)
    pages = torch.full((3, 32, max(rp, 32)), 7.0, dtype=dtype, device="cuda")
    slots = torch.tensor([33, 95, -1, 64, 40, 63], dtype=torch.int32)
    cq = latent_norm(z.cuda(), oq, wq.cuda(), 192, oc, wc.cuda() if nc else None, pages if nc else None, slots.cuda(),
                     eps)
    close(cq[:, :nq], O.rms_norm(z[:, oq:oq + nq].double(), wq.double(), eps), TOL[dt])
    assert (cq[:, nq:] == 0).all()
    flat = pages.view(-1, pages.shape[2]).cpu()
    keep = torch.ones(96, dtype=torch.bool)
    if nc:
        ref = O.rms_norm(z[:, oc:oc + nc].double(), wc.double(), eps)
        for t, s in enumerate(slots.tolist()):
            if s >= 0:
                close(flat[s, :nc], ref[t], TOL[dt])
                assert (flat[s, nc:] == 0).all()
                keep[s] = False
    assert (flat[keep] == 7).all()  # nothing else is touched


@pytest.mark.parametrize("dt", ["bf16", "f32"])
@pytest.mark.parametrize("nt", [1, 17, 40, 130])
def test_head_proj(dt, nt):
    from kgs.ops.latent import head_proj

    dtype, H, N, K, R = DT[dt], 3, 96, 64, 150
    a, w = rnd(R, H * K + 8, dtype=dtype), rnd(H, N, K, seed=1, dtype=dtype)
    gate = rnd(R, 64, seed=2, dtype=dtype)
    rows = torch.from_numpy(np.random.default_rng(nt).permutation(R)[:nt].astype(np.int32))
    ref = torch.einsum("rhk,hnk->rhn", a[:, :H * K].reshape(R, H, K).double(), w.double())
    out = torch.zeros(nt, H * N, dtype=dtype, device="cuda")
    head_proj(a.cuda()[:, :H * K], w.cuda(), nt, out, rows_in=rows.cuda())
    close(out, ref[rows.long()].reshape(nt, -1), TOL[dt])
    out = torch.zeros(R, H * N, dtype=dtype, device="cuda")
    head_proj(a.cuda()[:, :H * K], w.cuda(), nt, out, rows_out=rows.cuda(), gate=gate.cuda()[:, 4:])
    want = torch.zeros(R, H, N, dtype=torch.float64)
    want[rows.long()] = ref[:nt] * torch.sigmoid(gate[rows.long(), 4:4 + H].double())[:, :, None]
    close(out, want.reshape(R, -1), TOL[dt])


def run_latent(q, c, lens, n, H, scale, dt, nsplit=None):
    """q [sum n, H, R], c [B][len, R]: the last n[b] positions of each sequence."""
    from kgs.ops.latent import LatentRows, latent_attention, padded_latent, split_count, waves_for
    from kgs.serve.hybrid import Geometry, HostPack

    R, rp = q.shape[2], padded_latent(q.shape[2])
    lens, n = np.asarray(lens), np.asarray(n)
    W = int(-(-lens.max() // 32)) + 1
    bt, npages = pages_for(lens, W)
    pages = torch.full((npages, 32, rp), 3.0, dtype=DT[dt])  # what a reused page holds must not matter
    flat = pages.view(-1, rp)
    for b, x in enumerate(c):
        flat[slots_of(bt, b, np.arange(len(x)))] = torch.nn.functional.pad(x, (0, rp - R)).to(DT[dt])
    pos0 = lens - n
    row0 = np.cumsum(n) - n
    seq = np.repeat(np.arange(len(n)), n)
    pos = pos0[seq] + np.arange(n.sum()) - row0[seq]
    pk = HostPack(torch.device("cuda"))
    refs = [None] * 7 + [pk.add(bt), None]
    (r, shape), _ = Geometry(H, rp, 0).lay_out(pk, row0, n, pos0, bt, seq, pos, refs)
    get = pk.send()
    if nsplit:
        shape["nsplit"] = nsplit
    rows = LatentRows(**{k: None if v is None else get(v) for k, v in r.items()}, **shape)
    qp = torch.nn.functional.pad(q, (0, rp - R)).to(DT[dt]).reshape(len(seq), H * rp).cuda()
    o = latent_attention(qp, pages.cuda(), rows, H, scale)
    return o.reshape(len(seq), H, rp)[:, :, :R]


def ref_latent(q, c, lens, n, scale, dt):
    out, at = [], 0
    for b, x in enumerate(c):
        x = x.to(DT[dt]).double()
        for i in range(n[b]):
            vis = x[:lens[b] - n[b] + i + 1]
            s = torch.einsum("hr,jr->hj", q[at + i].to(DT[dt]).double(), vis) * scale
            out.append(torch.softmax(s, -1) @ vis)
        at += n[b]
    return torch.stack(out)


@pytest.mark.parametrize("dt", ["bf16", "f32"])
@pytest.mark.parametrize("R,H,nsplit", [(32, 1, None), (56, 5, 1), (72, 17, 3), (96, 4, None), (128, 40, 2),
                                        (180, 3, None), (250, 130, None), (384, 16, 5), (512, 33, None), (600, 2, 1)])
def test_latent_attention_ragged(dt, R, H, nsplit):
    """Portions of one to 45 tokens and decoded tokens, across page borders, with and
    without context splits."""
    lens, n = [1, 31, 32, 33, 64, 200, 45, 321], [1, 2, 32, 3, 1, 1, 45, 7]
    q = rnd(sum(n), H, R, scale=1.5)
    c = [rnd(m, R, seed=i + 1) for i, m in enumerate(lens)]
    got = run_latent(q, c, lens, n, H, R ** -0.5, dt, nsplit)
    close(got, ref_latent(q, c, lens, n, R ** -0.5, dt), 1.2e-2 if dt == "bf16" else 5e-6)


@pytest.mark.parametrize("dt", ["bf16", "f32"])
def test_latent_attention_sees_exactly_its_keys(dt):
    """One key stands out by 40 in score: at every border it is seen if and only if
    it is not ahead of the query."""
    R, H, L = 64, 2, 330
    d = torch.nn.functional.normalize(rnd(R, seed=3), dim=0)
    base = 0.05 * rnd(L, R, seed=4)
    q = (d[None, None] * 10).repeat(9, H, 1)
    for key in (0, 1, 30, 31, 32, 33, 63, 64, 255, 256, 257, 318, 321, 322, 323, 328, 329):
        c = base.clone()
        c[key] = 4 * d
        got = run_latent(q, [c], [L], [9], H, 1.0, dt, nsplit=4 if key % 2 else None).cpu().float()
        for i in range(9):
            sees = key <= L - 9 + i
            share = float(got[i, 0] @ d) / 4
            assert (share > 0.97) if sees else (share < 0.1), (key, i, share)


@pytest.mark.parametrize("hd", [64, 128])
def test_attention_ragged(hd):
    """The expanded form: portions of any length at any position, several in one
    launch, keys beyond and rows between them untouched, with the output gate."""
    from kgs.ops.transformer import attention_ragged

    H, scale = 3, 0.17
    lens, n = [300, 129, 64, 77, 513], [300, 129, 1, 70, 130]
    T, C = sum(n) + 5, sum(lens)
    q = rnd(T, H * hd, scale=1.2, dtype=torch.bfloat16)
    kv = rnd(C, 2 * H * hd, seed=1, dtype=torch.bfloat16)
    gate = rnd(T, 64, seed=2, dtype=torch.bfloat16)
    row, base, items, ref = 5, 0, [], torch.full((T, H, hd), 9.0, dtype=torch.float64)
    for L, m in zip(lens, n):
        for i in range(0, m, 128):
            items.append([row + i, base, L - m + i, min(128, m - i)])
        k, v = (x.reshape(L, H, hd).double() for x in kv[base:base + L].chunk(2, 1))
        s = torch.einsum("thd,jhd->htj", q[row:row + m].reshape(m, H, hd).double(), k) * scale
        s = s.masked_fill(torch.arange(L)[None] > (L - m + torch.arange(m))[:, None], float("-inf"))
        ref[row:row + m] = torch.einsum("htj,jhd->thd", torch.softmax(s, -1), v) * \
            torch.sigmoid(gate[row:row + m, :H].double())[:, :, None]
        row, base = row + m, base + L
    out = torch.full((T, H * hd), 9.0, dtype=torch.bfloat16, device="cuda")
    kvd = kv.cuda()
    attention_ragged(q.cuda(), kvd[:, :H * hd], kvd[:, H * hd:], torch.tensor(items, dtype=torch.int32).cuda(), H, hd,
                     scale, out, gate=gate.cuda())
    close(out.reshape(T, H, hd)[5:], ref[5:], 1.5e-2)
    assert (out[:5] == 9).all()


# ------------------------------------------------------------------- delta rule
class DeltaCase:
    def __init__(self, H, G, K, V, taps, T, seed=0, dtype=torch.float32, r=10, slots=4):
        from kgs.ops.delta import DeltaShape, DeltaState

        self.H, self.G, self.K, self.V, self.dtype = H, G, K, V, dtype
        self.sh = DeltaShape(H, G, K, V, taps)
        gk, hv = G * K, H * V
        self.offs = (8, 8 + gk, 16 + 2 * gk, 16 + 2 * gk + hv)
        self.z = rnd(T, self.offs[3] + H + 3, seed=seed, dtype=dtype)
        self.a2 = rnd(T, H * K + 1, seed=seed + 1, dtype=dtype)
        self.cw = rnd(taps, self.sh.channels, seed=seed + 2)
        self.a_log, self.dt_bias = rnd(H, seed=seed + 3) - 1, 2 * rnd(H * K, seed=seed + 4) - 2
        self.state = DeltaState(self.sh, slots, "cuda")
        self.state.S.fill_(5.0)  # a slot that was used before
        self.state.conv.fill_(5.0)

    def run(self, portions):
        """portions: per call a list of (first row, rows, position, slot); rows of a
        call are gathered into one batch. Returns o by row."""
        from kgs.ops.delta import RaggedSeqs, chunk_plan, delta_forward

        i32 = lambda a: torch.tensor(a, dtype=torch.int32, device="cuda")  # noqa: E731
        out = torch.zeros(self.z.shape[0], self.H, self.V)
        for call in portions:
            rows = torch.cat([torch.arange(a, a + n) for a, n, _, _ in call])
            n = [c[1] for c in call]
            row0 = [sum(n[:i]) for i in range(len(n))]
            seqs = RaggedSeqs(i32([b for b, m in enumerate(n) for _ in range(m)]), i32(row0), i32(n),
                              i32([c[2] for c in call]), i32([c[3] for c in call]),
                              **{k: i32(v.tolist()).reshape(v.shape) for k, v in chunk_plan(row0, n, [c[2] for c in call],
                                                                                        [c[3] for c in call]).items()})
            o = delta_forward(self.z[rows].cuda(), self.offs, self.a2[rows].cuda(), self.cw.cuda(), self.a_log.cuda(),
                              self.dt_bias.cuda(), self.sh, self.state, seqs)
            out[rows] = o.cpu()
        return out

    def ref(self, a, n):
        """Oracle of rows a .. a + n - 1 as one sequence: (o, final state)."""
        H, G, K, V = self.H, self.G, self.K, self.V
        z = self.z[a:a + n].double()
        oq, ok, ov, ob = self.offs
        cw = self.cw.double().T
        q, k = (O.silu(O.short_conv(z[:, o:o + G * K], cw[i * G * K:(i + 1) * G * K])).reshape(n, G, K)
                for i, o in enumerate((oq, ok)))
        v = O.silu(O.short_conv(z[:, ov:ov + H * V], cw[2 * G * K:])).reshape(n, H, V)
        q = (O.unit(q) * K ** -0.5).repeat_interleave(H // G, 1)
        k = O.unit(k).repeat_interleave(H // G, 1)
        x = (self.a2[a:a + n, :H * K].double() + self.dt_bias.double()).reshape(n, H, K)
        g = torch.exp(-torch.exp(self.a_log.double())[None, :, None] * O.softplus(x))
        return O.delta_rule(q, k, v, g, torch.sigmoid(z[:, ob:ob + H]))


SHAPES = [(1, 1, 32, 32, 1), (2, 2, 32, 32, 4), (6, 2, 20, 28, 3), (3, 3, 36, 12, 2), (4, 2, 64, 64, 4),
          (2, 1, 130, 70, 5), (4, 4, 8, 33, 4), (2, 1, 128, 128, 4), (1, 1, 256, 40, 4)]


@pytest.mark.parametrize("dt", ["bf16", "f32"])
@pytest.mark.parametrize("shape", SHAPES)
def test_delta_portions_equal_the_whole(dt, shape):
    """A prompt whole, in portions of 1, 2, 3 and more tokens, and token by token."""
    T = 41
    c = DeltaCase(*shape, T, dtype=DT[dt])
    ref, S = c.ref(0, T)
    for cut in ([T], [1] * T, [2, 2, 1, 3, 8, 9, 16], [17, 1, 1, 2, 20], [32, 9], [15, 26]):
        at, calls = 0, []
        for n in cut:
            calls.append([(at, n, at, 2)])
            at += n
        close(c.run(calls), ref, 3e-5)
        close(c.state.S[2, :, :, :c.K].transpose(1, 2), S, 3e-5)
    assert (c.state.S[2, :, :, c.K:] == 0).all() or c.K == c.sh.kp
    assert (c.state.S[1] == 5).all() and (c.state.conv[3] == 5).all()  # other slots are left alone


@pytest.mark.parametrize("shape", SHAPES[2:5])
def test_delta_ragged_batches_and_reused_slots(shape):
    c = DeltaCase(*shape, 150)
    a, b, d = (0, 70), (70, 45), (115, 35)
    calls = [[(0, 60, 0, 1), (70, 2, 0, 3)], [(72, 40, 2, 3)], [(60, 1, 60, 1), (112, 3, 42, 3)],
             [(61, 9, 61, 1), (115, 1, 0, 3)],   # slot 3 belongs to the next sequence now
             [(116, 34, 1, 3)]]
    o = c.run(calls)
    for lo, n in (a, b, d):
        close(o[lo:lo + n], c.ref(lo, n)[0], 3e-5)


def test_delta_decay_extremes():
    """Channels that forget at once beside channels that keep everything for long."""
    c = DeltaCase(2, 1, 64, 32, 4, 600)
    c.a_log = torch.tensor([3.0, 0.0])
    c.dt_bias = torch.where(torch.arange(128) % 2 == 0, 8.0, -12.0)
    close(c.run([[(0, 300, 0, 1)], [(300, 300, 300, 1)]]), c.ref(0, 600)[0], 5e-5)


@pytest.mark.parametrize("dt", ["bf16", "f32"])
def test_delta_out(dt):
    from kgs.ops.delta import delta_out

    T, H, V, ld = 5, 3, 28, 128
    o, w, gate = rnd(T, H, V), 1 + 0.1 * rnd(V, seed=1), rnd(T, H * V + 12, seed=2, dtype=DT[dt])
    y = delta_out(o.cuda(), w.cuda(), gate.cuda(), 1e-3, ld)
    ref = O.rms_norm(o.double(), w.double(), 1e-3) * torch.sigmoid(gate[:, :H * V].double()).reshape(T, H, V)
    close(y[:, :H * V], ref.reshape(T, -1), TOL[dt])
    assert (y[:, H * V:] == 0).all()
