"""Vumalix without a GPU: configuration and checkpoint reading, the registry, launch plans,
weight layouts, and the oracle itself."""
import json
import math
import os
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import vumalix_models as VM  # noqa: E402
from oracles import vumalix as O  # noqa: E402

from kgs.models.registry import from_spec, load_config, of_config, to_spec  # noqa: E402
from kgs.models.ruruzen import LatentSpec  # noqa: E402
from kgs.models.vumalix import DiffAttentionSpec, VumalixConfig, check_weights, tensor_shapes  # noqa: E402
from kgs.ops.latent import padded_latent, padded_rot, window_pages  # noqa: E402
from kgs.ops.paged import paged_heads, row_splits, tile_queries  # noqa: E402
from kgs.ops.postnorm import Conv, ConvState  # noqa: E402
from kgs.serve.hybrid import Geometry, neighbours  # noqa: E402
from kgs.serve.ragged import HostPack  # noqa: E402
from kgs.utils.safetensors import save_file  # noqa: E402

BF = torch.bfloat16


# ------------------------------------------------------------ configuration
def test_config_reads_every_size():
    c = VM.config("mixed")
    assert (c.vocab, c.width, c.eps, c.taps) == (203, 140, 3e-6, 4)
    assert c.layers[0].mixer == LatentSpec(3, 24, 40, 36, 56, 0.25, rot_dim=8, rot_base=1e3, window=20, gate_each=True)
    assert c.layers[1].mixer == DiffAttentionSpec(4, 2, 24, 40, 0.2, 0.3, 0.5, 7)
    assert [x.ff for x in c.layers] == [72, 100, 72, None, 100, 72]
    assert [x.owner for x in c.layers] == [0, 1, 0, 3, 1, 0] and c.owners == [0, 1, 3]
    assert VM.config("large").owners == [0, 2, 3]  # layer 1 uses a later one's
    d = json.loads(json.dumps(c.raw))
    d["layers"][5]["weights_of"] = 2  # which uses layer 0's
    assert VumalixConfig.from_dict(d).layers == c.layers
    d["layers"][5]["mixer"].pop("mask")
    d["layers"][5].pop("weights_of")
    assert VumalixConfig.from_dict(d).layers[5].mixer.window == 0
    assert c.has_state and not VM.config("stateless").has_state


@pytest.mark.parametrize("change", [
    lambda d: d.update(architecture="Llama"),
    lambda d: d["layers"][0].update(type="window"),
    lambda d: d["layers"][0].update(mixer=None),
    lambda d: d["layers"][0]["mixer"]["rot"].update(dims=4),
    lambda d: d["layers"][0]["mixer"].update(rot_dim=7),
    lambda d: d["layers"][0]["mixer"]["rot"].update(base=0),
    lambda d: d["layers"][0]["mixer"]["mask"].update(size=0),
    lambda d: d["layers"][0]["mixer"].update(kv_rank=0),
    lambda d: d["layers"][1]["mixer"].update(kv_heads=3),
    lambda d: d["layers"][1]["mixer"].update(scale=None),
    lambda d: d["layers"][1]["mixer"].update(scale=0),
    lambda d: d["layers"][1]["mixer"].update(diff="a"),
    lambda d: d["layers"][1]["mixer"]["q_temp"].update(every=0),
    lambda d: d["layers"][1]["mixer"]["q_temp"].pop("coef"),
    lambda d: d["layers"][0]["mlp"].update(kind="gelu"),
    lambda d: d["layers"][0]["mlp"].update(ff=0),
    lambda d: d["layers"][2].update(weights_of=6), lambda d: d["layers"][2].update(weights_of=1),
    lambda d: d["layers"][0].update(weights_of=2), lambda d: d["layers"][2].update(mlp=None),
    lambda d: d["canon"].update(taps=0), lambda d: d["norm"].pop("eps"),
    lambda d: d.update(width=0), lambda d: d.update(layers=[]),
])
def test_config_refuses_what_it_cannot_mean(change):
    d = json.loads(json.dumps({"architecture": "Vumalix", **VM.MODELS["mixed"]}))
    change(d)
    with pytest.raises(ValueError):
        VumalixConfig.from_dict(d)


def test_registry_and_checkpoint_roundtrip(tmp_path):
    cfg, w = VM.model("mixed")
    (tmp_path / "config.json").write_text(json.dumps(cfg.raw))
    save_file(w, tmp_path / "model.safetensors")
    c = load_config(tmp_path)
    assert of_config(c).name == "Vumalix" and c.layers == cfg.layers and c.path == str(tmp_path)
    got = c.load_weights()
    assert set(got) == set(w) and all(torch.equal(got[k], w[k]) for k in w)
    assert got["l0.norm1"].shape == ()
    assert from_spec(json.loads(json.dumps(to_spec(c)))) == c  # what a replica process gets
    from kgs.serve.vumalix import VumalixModel

    assert of_config(c).serving_class() is VumalixModel


def test_checkpoint_shapes_are_checked():
    cfg, w = VM.model("mixed")
    check_weights(cfg, w)
    for name in ("l0.mix.dkv", "l0.canon1", "l1.mix.q.norm", "l1.mix.lk2", "l0.mlp.act", "head"):
        bad = dict(w)
        bad[name] = w[name][..., :-1]
        with pytest.raises(ValueError, match=name.replace(".", r"\.")):
            check_weights(cfg, bad)
    with pytest.raises(ValueError, match="l0.norm1"):
        check_weights(cfg, {**w, "l0.norm1": torch.ones(140)})
    s = tensor_shapes(cfg)
    assert s["l0.mix.uq"] == (3 * 32, 36) and s["l0.mix.dkv"] == (64, 140) and s["l1.mix.k"] == (2 * 2 * 24, 140)
    assert "l3.norm2" not in s and not any(n.startswith(("l2.", "l4.", "l5.")) for n in s)


def test_memory_counts_every_layer():
    """Layers with another one's weights have cache and state of their own."""
    from kgs.serve.vumalix import VumalixModel, attention_heads

    cfg = VM.config("mixed")
    m = VumalixModel.memory(cfg, "bfloat16", 3)
    assert m["state"] == 4 * 6 * ConvState.bytes_per_slot(4, 256) == 4 * 6 * 3 * 256 * 4
    a, b = (attention_heads(cfg.layers[i].mixer, BF) for i in (1, 3))
    assert (a.dkp, a.dvp, a.maps, b.dkp) == (128, 64, 2, 128)
    assert m["page"] == 32 * 2 * (3 * (64 + 32) + 2 * 2 * (128 + 64) + 5 * (128 + 64))
    assert VumalixModel.memory(VM.config("stateless"), "bfloat16", 3)["state"] == 0


# ---------------------------------------------------------------------- plans
def test_head_forms():
    h = paged_heads(12, 3, 100, 64, BF, maps=2)
    assert (h.dkp, h.dvp, h.mfma, tile_queries(h)) == (256, 64, True, 16)
    assert tile_queries(paged_heads(40, 1, 40, 100, BF, maps=2)) == 1
    assert tile_queries(paged_heads(80, 1, 64, 64, BF, maps=2)) == 0  # a group larger than a tile
    assert not paged_heads(4, 2, 160, 32, BF, maps=2).mfma and paged_heads(4, 2, 160, 32, BF, maps=2).dkp == 320
    assert row_splits(1, 8, 4, 300, maps=2) == row_splits(1, 8, 4, 300) and row_splits(8, 8, 12, 300, 2) < row_splits(8, 8, 12, 300)
    assert (padded_rot(2), padded_rot(32), padded_rot(33), padded_latent(130)) == (32, 32, 64, 192)
    with pytest.raises(ValueError):
        padded_rot(600)


def test_window_pages():
    """The most pages that any run of query tokens sees, counted out."""
    for window in (1, 2, 31, 32, 33, 34, 64, 65, 100):
        for n in (1, 2, 5, 33):
            most = max((p + n - 1) // 32 - max(0, p - window + 1) // 32 + 1 for p in range(400))
            assert window_pages(window, n) == most, (window, n)


def _lay_out(geo, n, pos0):
    n, pos0 = np.array(n), np.array(pos0)
    row0 = np.cumsum(n) - n
    seq = np.repeat(np.arange(len(n)), n)
    pos = pos0[seq] + np.arange(n.sum()) - row0[seq]
    bt = 100 * np.arange(len(n))[:, None] + np.arange(40)
    pk = HostPack(torch.device("cpu"))
    refs = [None] * 7 + [pk.add(bt), None]
    plan = geo.host_plan(pk, row0, n, pos0, bt, seq, pos, refs)
    return plan(pk.send())


def test_expanded_portions_hold_only_their_window():
    p = _lay_out(Geometry(4, 128, 64, 50), [200, 3, 1], [100, 7, 900])
    e = p.expanded
    first = 100 - 50 + 1
    assert e.ctx_slots.tolist() == [(x // 32) * 32 + x % 32 for x in range(first, 300)]
    assert sorted(e.items.tolist()) == [[0, 0, 49, 128], [128, 0, 177, 72]]
    assert p.absorbed.nt == 4 and p.absorbed.tok_pos.tolist() == [7, 8, 9, 900]
    assert p.absorbed.nsplit <= window_pages(50, 3 * 16)
    whole = _lay_out(Geometry(4, 128, 64), [200, 3, 1], [100, 7, 900]).expanded
    assert whole.ctx_slots.numel() == 300 and sorted(whole.items.tolist()) == [[0, 0, 100, 128], [128, 0, 228, 72]]


def test_expansion_counts_the_window():
    g, far = Geometry(8, 512, 128, 64), Geometry(8, 512, 128)
    # 40 tokens far into a long context: the whole of it is too much to expand, a window is not
    assert not far.expand(40, 100000) and g.expand(200, 100000) and not g.expand(16, 100000)
    assert g.expand(100, 0) == far.expand(100, 0) and Geometry(8, 512, 128, 10**6).expand(40, 500) == far.expand(40, 500)


def test_rotated_halves_become_neighbours():
    t = torch.arange(12.0).reshape(6, 2)
    assert neighbours(t, 0)[:, 0].tolist() == [0, 6, 2, 8, 4, 10]
    assert torch.equal(neighbours(t[None], 1)[0], neighbours(t, 0))


def test_convolution_weights_are_turned_around():
    w = torch.arange(6.0).reshape(2, 3)
    c = Conv(w, 8)
    assert c.taps == 3 and c.w[:, :2].tolist() == [[2.0, 5.0], [1.0, 4.0], [0.0, 3.0]] and (c.w[:, 2:] == 0).all()


# --------------------------------------------------------------------- oracle
def test_oracle_mechanisms():
    """Each mechanism against its definition written out."""
    g = torch.Generator().manual_seed(3)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    x, w = r(5, 3), r(3, 3)
    y = O.causal_conv(x, w)
    assert torch.allclose(y[4, 1], w[1, 2] * x[4, 1] + w[1, 1] * x[3, 1] + w[1, 0] * x[2, 1])
    assert torch.allclose(y[1, 0], w[0, 2] * x[1, 0] + w[0, 1] * x[0, 0]) and torch.allclose(y[0], w[:, 2] * x[0])
    q = r(5, 2, 6)
    t, a = O.rotate_half(q, 9.0), 3 * 9.0 ** (-2 / 6)
    assert torch.allclose(t[3, 1, 1], q[3, 1, 1] * math.cos(a) - q[3, 1, 4] * math.sin(a))
    assert torch.allclose(t[3, 1, 4], q[3, 1, 4] * math.cos(a) + q[3, 1, 1] * math.sin(a)) and torch.equal(t[0], q[0])
    m = O.window_mask(6, 3)
    assert m[5].tolist() == [False, False, False, True, True, True] and m[1].tolist() == [True, True] + [False] * 4
    assert O.temperature(8, {"coef": 0.5, "every": 3}, torch.float64).tolist() == \
        [1, 1] + [1 + 0.5 * math.log(2)] * 3 + [1 + 0.5 * math.log(3)] * 3
    z, act = r(4, 7), torch.tensor([0.3, -0.4, 0.5, 0.2], dtype=torch.float64)
    n = lambda u: u / ((u * u).mean() + 0.1).sqrt()  # noqa: E731
    assert torch.allclose(O.poly_norm(z, act, 0.1)[2], 0.3 * n(z[2]) - 0.4 * n(z[2] ** 2) + 0.5 * n(z[2] ** 3) + 0.2)
    ws = {k: r(4) for k in ("lq1", "lk1", "lq2", "lk2")}
    assert torch.allclose(O.mixing_lambda(ws, "", 0.6), torch.exp(ws["lq1"] @ ws["lk1"]) - torch.exp(ws["lq2"] @ ws["lk2"]) + 0.6)


def test_oracle_differential_attention_written_out():
    cfg, w = VM.model("mixed")
    m, p = cfg.raw["layers"][1]["mixer"], "l1.mix."
    w = {n: t.double() for n, t in w.items()}
    h = torch.randn(9, 140, generator=torch.Generator().manual_seed(1), dtype=torch.float64)
    got = O.differential_attention(h, w, p, m, 1e-3)
    t, out = 8, []
    lam = O.mixing_lambda(w, p, m["diff"])
    n = lambda u: u / ((u * u).mean() + 1e-3).sqrt()  # noqa: E731
    for head in range(4):
        kv, maps = head // 2, []
        for i in range(2):
            rows = slice((2 * head + i) * 24, (2 * head + i + 1) * 24)
            q = n(w[p + "q"][rows] @ h[t]) * w[p + "q.norm"] * (1 + 0.5 * math.log(9 // 7 + 1))
            s = torch.stack([q @ (n(w[p + "k"][(2 * kv + i) * 24:(2 * kv + i + 1) * 24] @ x) * w[p + "k.norm"]) for x in h]) * 0.2
            maps.append(torch.softmax(s, 0) @ (h @ w[p + "v"][40 * kv:40 * kv + 40].T))
        out.append(n(maps[0] - lam * maps[1]) * 0.7)
    assert torch.allclose(got[t], w[p + "o"] @ torch.cat(out))


def test_oracle_planted_mistakes_show():
    """Each mistake in the oracle moves the logits by far more than rounding: the test
    models are sensitive to what the GPU tests check."""
    toks = np.random.default_rng(0).integers(0, 203, size=60).tolist()
    cfg, w = VM.model("mixed")
    base = O.forward(cfg.raw, w, toks)

    def run(patch=None, weights=None, change=None):
        raw = json.loads(json.dumps(cfg.raw))
        if change:
            change(raw)
        saved = {n: getattr(O, n) for n in patch or {}}
        try:
            for n, f in (patch or {}).items():
                setattr(O, n, f)
            d = O.forward(raw, weights or w, toks) - base
        finally:
            for n, f in saved.items():
                setattr(O, n, f)
        return float(d.pow(2).mean().sqrt() / base.std())

    mask, turn, conv, temp, lam, poly = O.window_mask, O.rotate_half, O.causal_conv, O.temperature, O.mixing_lambda, O.poly_norm
    split = lambda x, w: torch.cat([conv(x[:30], w), conv(x[30:], w)])  # noqa: E731
    assert run() == 0
    assert run({"window_mask": lambda T, s: mask(T, s + 1 if s == 20 else s)}) > 1e-2
    assert run({"window_mask": lambda T, s: mask(T, T)}) > 1e-2
    assert run({"rotate_half": lambda x, b: x}) > 1e-2
    assert run({"rotate_half": lambda x, b: turn(x.flip(-1), b).flip(-1)}) > 1e-2
    assert run({"causal_conv": split}) > 1e-2
    assert run({"causal_conv": lambda x, w: conv(x, w.flip(1))}) > 1e-2
    assert run({"temperature": lambda T, m, d: temp(T + 1, m, d)[1:]}) > 1e-3
    assert run({"temperature": lambda T, m, d: temp(T, m, d) * 0 + 1}) > 1e-2
    assert run({"mixing_lambda": lambda w, p, d: lam(w, p, 0 * d)}) > 1e-2
    assert run({"poly_norm": lambda z, a, e: poly(z, torch.stack([a[0], a[1], a[2], 0 * a[3]]), e)}) > 1e-3
    assert run({"poly_norm": lambda z, a, e: poly(z, torch.stack([a[0], a[2], a[1], a[3]]), e)}) > 1e-2
    assert run(weights={**w, "l0.mix.g": 0 * w["l0.mix.g"]}) > 1e-2
    assert run(weights={**w, "l1.norm2": w["l1.norm2"] * 1.1}) > 1e-2
    assert run(change=lambda d: d["layers"][1]["mixer"].update(diff=0.31)) > 1e-4
