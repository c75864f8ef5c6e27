"""Nokipel without a GPU: configuration and checkpoint reading, the registry, launch
plans, decay and rotary tables, and the oracle itself."""
import json
import math
import os
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import nokipel_models as NM  # noqa: E402
from oracles import nokipel as O  # noqa: E402

from kgs.models.nokipel import AttentionSpec, DenseSpec, ExpertsSpec, LightningSpec, NokipelConfig, check_weights, tensor_shapes  # noqa: E402
from kgs.models.registry import from_spec, load_config, of_config, to_spec  # noqa: E402
from kgs.ops.lightning import Decays, LightningShape, segment_plan  # noqa: E402
from kgs.ops.paged import paged_heads, portion_items, row_splits, tile_queries, visible_pages  # noqa: E402
from kgs.ops.talking import Rotary  # noqa: E402
from kgs.utils.safetensors import save_file  # noqa: E402

BF = torch.bfloat16


# ------------------------------------------------------------ configuration
def test_config_reads_every_size():
    c = NM.config("mixed")
    assert (c.vocab, c.width, c.eps, c.norm_groups, c.embed_scale, c.loop) == (203, 140, 3e-6, 5, 3.5, (1, 3, 3))
    assert c.layers[0].mixer == LightningSpec(4, 24, 40, (0.5, 0.9, 0.98, 0.9995)) and c.layers[0].mlp == DenseSpec(72, 0.8)
    assert c.layers[1].mixer == AttentionSpec(4, 2, 24, 40, 0.3, 20, 12, 1e3)
    assert c.layers[1].mlp == ExpertsSpec(5, 1, 3, 3, 2, 1.3, 48, 56)
    assert c.layers[2].mlp == ExpertsSpec(7, 0, 3, 1, 1, 1.0, 40, 0) and c.layers[3].mlp is None
    assert c.has_state and not NM.config("stateless").has_state


def test_layer_runs():
    assert NM.config("mixed").runs == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False), (3, False)]
    assert NM.config("first").runs == [(0, False), (1, False), (0, True), (1, False)]
    assert NM.config("large").runs == [(0, False), (1, False), (2, False), (3, False), (3, True), (3, True)]
    assert NM.config("stateless").runs == [(0, False), (1, False), (2, False)]
    for n in NM.MODELS:
        assert NM.config(n).runs == O.order(NM.config(n).raw)


@pytest.mark.parametrize("change", [
    lambda d: d.update(architecture="Llama"),
    lambda d: d["layers"][0].update(type="window"),
    lambda d: d["layers"][0].update(mixer=None),
    lambda d: d["layers"][0]["mixer"].update(decay=[0.5]),
    lambda d: d["layers"][0]["mixer"].update(decay=["a"] * 4),
    lambda d: d["layers"][1]["mixer"].update(kv_heads=3),
    lambda d: d["layers"][1]["mixer"].update(scale=None),
    lambda d: d["layers"][1]["mixer"].update(scale=0),
    lambda d: d["layers"][1]["mixer"]["rot"].update(dims=13),
    lambda d: d["layers"][1]["mixer"]["rot"].update(dims=26),
    lambda d: d["layers"][1]["mixer"]["mask"].update(size=0),
    lambda d: d["layers"][0]["mlp"].update(kind="gelu"),
    lambda d: d["layers"][0]["mlp"].pop("limit"),
    lambda d: d["layers"][1]["mlp"]["router"].update(top=5),
    lambda d: d["layers"][1]["mlp"]["router"].update(identity=-1),
    lambda d: d["layers"][1]["mlp"]["router"]["groups"].update(count=4),
    lambda d: d["layers"][1]["mlp"]["router"]["groups"].update(keep=4),
    lambda d: d["layers"][1]["mlp"]["expert"].update(ff=0),
    lambda d: d["loop"].update(stop=5), lambda d: d["loop"].update(start=3), lambda d: d["loop"].update(times=0),
    lambda d: d["norm"].update(groups=3), lambda d: d.update(width=0), lambda d: d.update(layers=[]),
])
def test_config_refuses_what_it_cannot_mean(change):
    d = json.loads(json.dumps({"architecture": "Nokipel", **NM.MODELS["mixed"]}))
    change(d)
    with pytest.raises(ValueError):
        NokipelConfig.from_dict(d)


def test_registry_and_checkpoint_roundtrip(tmp_path):
    cfg, w = NM.model("mixed")
    (tmp_path / "config.json").write_text(json.dumps(cfg.raw))
    save_file(w, tmp_path / "model.safetensors")
    c = load_config(tmp_path)
    assert of_config(c).name == "Nokipel" and c.layers == cfg.layers and c.path == str(tmp_path)
    got = c.load_weights()
    assert set(got) == set(w) and all(torch.equal(got[k], w[k]) for k in w)
    assert from_spec(json.loads(json.dumps(to_spec(c)))) == c  # what a replica process gets
    from kgs.serve.nokipel import NokipelModel

    assert of_config(c).serving_class() is NokipelModel


def test_checkpoint_shapes_are_checked():
    cfg, w = NM.model("mixed")
    check_weights(cfg, w)
    for name in ("l0.mix.norm", "l1.mix.v.b", "l1.mlp.correction", "l1.mlp.e4.down", "l1.mlp.shared.sg", "l2.mix.g", "head"):
        bad = dict(w)
        bad[name] = w[name][..., :-1]
        with pytest.raises(ValueError, match=name.replace(".", r"\.")):
            check_weights(cfg, bad)
    del w["l2.norm2"]
    with pytest.raises(ValueError, match="l2.norm2"):
        check_weights(cfg, w)
    s = tensor_shapes(cfg)
    assert "l3.norm2" not in s and "l2.mlp.shared.sg" not in s and s["l1.mlp.router"] == (6, 140)


def test_memory_counts_every_run():
    from kgs.ops.lightning import LightningState
    from kgs.serve.nokipel import NokipelModel, attention_heads, lightning_shape

    cfg = NM.config("mixed")
    m = NokipelModel.memory(cfg, "bfloat16", 3)
    a, b = (LightningState.bytes_per_slot(lightning_shape(cfg.layers[i].mixer)) for i in (0, 2))
    assert m["state"] == 4 * (a + 3 * b)
    h1, h3 = (attention_heads(cfg.layers[i].mixer, BF) for i in (1, 3))
    assert m["page"] == 32 * 2 * (3 * h1.kv_heads * (h1.dkp + h1.dvp) + h3.kv_heads * (h3.dkp + h3.dvp))


# --------------------------------------------------------------------- tables
def test_decay_tables():
    d = Decays([0.0, 0.5, 0.9995, 1.0], "cpu")
    assert d.tokens.shape == (4, 65) and d.chunks.shape == (4, 65)
    assert d.tokens[0].tolist() == [1.0] + [0.0] * 64 and (d.tokens[3] == 1).all() and (d.chunks[3] == 1).all()
    assert d.chunks[0].tolist() == [1.0] + [0.0] * 64
    assert abs(float(d.tokens[2, 64]) - 0.9995 ** 64) < 1e-7 and abs(float(d.chunks[2, 60]) - 0.9995 ** (64 * 60)) < 1e-7


def test_rotary_table():
    t = Rotary(6, 100.0, 50, "cpu").table
    assert t.shape == (50, 8) and t[:, 6:].tolist() == [[1.0, 0.0]] * 50
    for p, i in ((0, 0), (7, 1), (49, 2)):
        a = p * 100.0 ** (-2 * i / 6)
        assert abs(float(t[p, 2 * i]) - math.cos(a)) < 1e-7 and abs(float(t[p, 2 * i + 1]) - math.sin(a)) < 1e-7


# ---------------------------------------------------------------------- plans
def test_head_forms():
    h = paged_heads(32, 8, 100, 64, BF)
    assert (h.dkp, h.dvp, h.mfma, tile_queries(h)) == (128, 64, True, 32)
    assert tile_queries(paged_heads(6, 2, 40, 24, BF)) == 42 and tile_queries(paged_heads(128, 1, 64, 64, BF)) == 1
    assert tile_queries(paged_heads(200, 1, 64, 64, BF)) == 0  # a group larger than a tile
    assert not paged_heads(4, 2, 160, 32, BF).mfma and not paged_heads(4, 2, 64, 64, torch.float32).mfma
    with pytest.raises(ValueError):
        paged_heads(2, 1, 64, 2000, BF)
    s = LightningShape(3, 100, 130)
    assert (s.kp, s.vp, s.slabs) == (128, 256, 2) and LightningShape(1, 8, 8).vp == 64
    with pytest.raises(ValueError):
        LightningShape(1, 300, 8)


def test_visible_pages_and_splits():
    assert [visible_pages(p, 0) for p in (0, 31, 32, 95)] == [1, 1, 2, 3]
    assert [visible_pages(p, 40) for p in (0, 39, 40, 79, 80, 119)] == [1, 2, 1, 2, 1, 2]
    assert visible_pages(47, 48) == 2 and visible_pages(48, 48) == 1 and visible_pages(95, 48) == 2
    for n, kv, g, pages in ((1, 8, 4, 300), (64, 8, 4, 32), (1000, 2, 1, 9), (3, 1, 40, 1)):
        s = row_splits(n, kv, g, pages)
        assert 1 <= s <= 64 and (s == 1 or (s - 1) * 8 < pages)


def _plan(heads, n, pos0, chunk):
    from kgs.serve.nokipel import ChunkedGeometry
    from kgs.serve.ragged import HostPack

    n, pos0 = np.array(n), np.array(pos0)
    row0 = np.cumsum(n) - n
    row_seq = np.repeat(np.arange(len(n)), n)
    pos = pos0[row_seq] + np.arange(n.sum()) - row0[row_seq]
    bt = np.arange(len(n) * 40).reshape(len(n), 40)
    pk = HostPack(torch.device("cpu"))
    refs = [pk.add(a) for a in (pos, pos, row_seq, row0, n, pos0, pos0, bt, pos, pos)]
    return ChunkedGeometry(heads, chunk).host_plan(pk, row0, n, pos0, bt, row_seq, pos, refs)(pk.send())


def test_attention_plan_splits_tiles_and_rows():
    h = paged_heads(12, 3, 64, 64, BF)  # 32 queries a tile
    p = _plan(h, [1, 40, 2, 16, 15], [70, 3, 9, 500, 0], 100)
    assert sorted(p.tiles.items.tolist()) == [[1, 1, 3, 32], [33, 1, 35, 8], [43, 3, 500, 16]]
    assert p.tiles.items.tolist()[-1] == [43, 3, 500, 16]  # the fewest keys: its chunk has just begun
    assert p.rows.n == 18 and p.rows.rows.tolist() == [0, 41, 42, *range(59, 74)]
    assert p.rows.tok_seq.tolist() == [0, 2, 2] + [4] * 15 and p.rows.tok_pos.tolist() == [70, 9, 10, *range(15)]
    p = _plan(h, [1, 1], [5, 900], 100)
    assert p.tiles is None and p.rows.rows is None and p.rows.tok_pos.tolist() == [5, 900]
    assert _plan(h, [64], [0], 0).rows is None
    p = _plan(paged_heads(4, 2, 160, 32, BF), [64], [0], 16)  # no tiled kernel for it
    assert p.tiles is None and p.rows.n == 64


def test_portion_items_cover_every_query_once():
    for tile in (1, 7, 32):
        items = portion_items([(0, 0, 5, 70), (70, 3, 0, 1), (71, 1, 900, 33)], tile, 48)
        got = sorted((r + j, s, p + j) for r, s, p, n in items.tolist() for j in range(n))
        assert got == [(i, 0, 5 + i) for i in range(70)] + [(70, 3, 0)] + [(71 + i, 1, 900 + i) for i in range(33)]
        assert items[:, 3].max() <= tile


def test_segment_plan():
    p = segment_plan([1, 15, 16, 200], 512)
    assert p["step"].tolist() == [0, 1] and p["items"].tolist() == [[3, 0, 200, -1], [2, 0, 16, -1]]
    assert p["scans"] == [] and p["buffers"] == 0
    p = segment_plan([3, 8192, 700], 32)  # 139 chunks of 32 workgroups: segments of 9 chunks
    assert p["step"].tolist() == [0] and [list(map(int, s)) for s in p["scans"]] == [[1, 0, 15, 9], [2, 15, 2, 9]]
    items = p["items"]
    for s, n in ((1, 8192), (2, 700)):
        it = items[items[:, 0] == s]
        it = it[np.argsort(it[:, 1])]
        assert (it[:-1, 2] == 9 * 64).all() and it[:, 2].sum() == n and (np.diff(it[:, 3]) == 1).all()
        assert it[:, 1].tolist() == [i * 9 * 64 for i in range(len(it))]
    assert p["buffers"] == 17 and (np.diff(items[:, 2]) <= 0).all()
    assert segment_plan([100, 5], 8, chunked=False)["step"].tolist() == [0, 1]
    long = segment_plan([300000], 64)  # never more than the decay table has
    assert long["scans"][0][3] <= 64


# --------------------------------------------------------------------- oracle
def test_oracle_mechanisms():
    """Each mechanism against its definition written out."""
    g = torch.Generator().manual_seed(3)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    x, w = r(3, 12), r(12)
    y = O.group_norm(x, w, 3, 0.5)
    assert torch.allclose(y[1, 6], x[1, 6] / ((x[1, 4:8] ** 2).mean() + 0.5).sqrt() * w[6])
    q = r(5, 2, 8)
    t = O.rotate(q, 4, 9.0)
    a = 3 * 9.0 ** (-2 / 4)
    assert torch.allclose(t[3, 1, 2], q[3, 1, 2] * math.cos(a) - q[3, 1, 3] * math.sin(a))
    assert torch.allclose(t[3, 1, 3], q[3, 1, 3] * math.cos(a) + q[3, 1, 2] * math.sin(a))
    assert torch.equal(t[..., 4:], q[..., 4:]) and torch.equal(t[0], q[0])
    m = O.chunk_mask(7, 3)
    assert m[5].tolist() == [False, False, False, True, True, True, False] and m[3].sum() == 1 and m[6].sum() == 1
    k, v = r(5, 2, 8), r(5, 2, 3)
    o = O.recurrence(q, k, v, [0.5, 0.25])
    want = sum(0.25 ** (4 - j) * (q[4, 1] @ k[j, 1]) * v[j, 1] for j in range(5))
    assert torch.allclose(o[4, 1], want)
    h, we = r(8), {"gate": 5 * r(12, 8), "up": 5 * r(12, 8), "down": r(8, 12)}
    gt, u = torch.clamp(we["gate"] @ h, max=0.7), torch.clamp(we["up"] @ h, -0.7, 0.7)
    assert gt.min() < -0.7 and torch.allclose(O.dense(h, we, "", 0.7), we["down"] @ (gt / (1 + torch.exp(-1.702 * gt)) * (u + 1)))
    z = we["gate"] @ h
    assert torch.allclose(O.expert(h, we, ""), we["down"] @ (z / (1 + torch.exp(-z)) * (we["up"] @ h)))


def test_oracle_routing():
    """Groups by their largest choice score; weights without the correction."""
    z = torch.log(torch.tensor([[0.3, 0.1, 0.25, 0.05, 0.2, 0.1]], dtype=torch.float64))
    eye, none = torch.eye(6, dtype=torch.float64), torch.zeros(6, dtype=torch.float64)
    cfg = {"top": 2, "scale": 2.0, "groups": {"count": 3, "keep": 1}}
    idx, w = O.route(z, eye, none, cfg)
    assert idx.tolist() == [[0, 1]] and torch.allclose(w, torch.tensor([[1.5, 0.5]], dtype=torch.float64))
    corr = torch.tensor([-1, -1, -1, -0.4, -1, -1], dtype=torch.float64)
    idx, w = O.route(z, eye, corr, cfg)
    assert idx.tolist() == [[3, 2]] and torch.allclose(w, torch.tensor([[1 / 3, 5 / 3]], dtype=torch.float64))
    idx, _ = O.route(z, eye, none, {"top": 2})
    assert idx.tolist() == [[0, 2]]


def test_oracle_planted_mistakes_show():
    """Each mistake in the oracle moves the logits by far more than rounding: the test
    models are sensitive to what the GPU tests check."""
    toks = np.random.default_rng(0).integers(0, 203, size=60).tolist()
    cfg, w = NM.model("mixed")
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

    mask, rotate, order, norm, rec, route = O.chunk_mask, O.rotate, O.order, O.group_norm, O.recurrence, O.route
    half = lambda x, dims, base: rotate(x.reshape(*x.shape[:-1], 2, -1).transpose(-1, -2).reshape(x.shape), dims, base)  # noqa: E731
    assert run() == 0
    assert run({"chunk_mask": lambda T, s: mask(T, s + 1)}) > 1e-2
    assert run({"chunk_mask": lambda T, s: torch.ones(T, T, dtype=torch.bool).tril()}) > 1e-2
    assert run({"rotate": half}) > 1e-2
    assert run({"order": lambda c: [(i, False) for i, _ in order(c)]}) > 1e-2
    assert run({"group_norm": lambda x, w, g, e: norm(x, w, 1, e)}) > 1e-2
    assert run({"recurrence": lambda q, k, v, d: torch.cat([rec(q[:30], k[:30], v[:30], d), rec(q[30:], k[30:], v[30:], d)])}) > 1e-2
    assert run({"route": lambda h, r, c, m: route(h, r, c * 0, m)}) > 1e-3
    assert run({"route": lambda h, r, c, m: route(h, r, c, {**m, "groups": None})}) > 1e-3
    assert run(weights={**w, "l1.mlp.shared.sg": 0 * w["l1.mlp.shared.sg"]}) > 1e-3
    assert run(weights={**w, "l1.mix.v.b": 0 * w["l1.mix.v.b"]}) > 1e-3
    assert run(change=lambda d: d["layers"][0]["mlp"].update(limit=8.0)) > 1e-3
    assert run(change=lambda d: d["layers"][0]["mixer"].update(decay=[0.5, 0.9, 0.98, 0.999])) > 1e-4
