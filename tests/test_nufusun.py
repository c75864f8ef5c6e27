"""Nufusun without a GPU: configuration and checkpoint reading, the registry, distance
buckets, layouts of the mixing matrix, launch plans, and the oracle itself."""
import json
import math
import os
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import nufusun_models as NM  # noqa: E402
from oracles import nufusun as O  # noqa: E402

from kgs.models.nufusun import NufusunConfig, check_weights, tensor_shapes  # noqa: E402
from kgs.models.registry import from_spec, load_config, of_config, to_spec  # noqa: E402
from kgs.ops.talking import TalkingWeights, buckets, heads_of, mix_fragments, tile_items  # noqa: E402
from kgs.utils.safetensors import save_file  # noqa: E402


# ------------------------------------------------------------ configuration
def test_config_reads_every_size():
    c = NM.config("mixed")
    assert (c.vocab, c.width, c.eps, c.embed_scale, len(c.layers)) == (203, 140, 3e-6, 3.5, 4)
    m, f = c.layers[0].mixer, c.layers[0].mlp
    assert (m.heads, m.kv_heads, m.dim, m.vdim, m.scale, m.bias_max) == (4, 2, 24, 40, 0.2, 20)
    assert (f.experts, f.top, f.ff, f.limit) == (5, 2, 48, 0.7)
    assert c.layers[1].mlp is None and c.layers[1].mixer.bias_max == 90.5


@pytest.mark.parametrize("change", [
    lambda d: d.update(architecture="Llama"),
    lambda d: d["layers"][0].update(type="window"),
    lambda d: d["layers"][0].update(mixer=None),
    lambda d: d["layers"][0]["mixer"].update(kv_heads=3),
    lambda d: d["layers"][0]["mixer"].update(scale=None),
    lambda d: d["layers"][0]["mlp"].update(kind="dense"),
    lambda d: d["layers"][0]["mlp"]["router"].update(top=6),
    lambda d: d["layers"][0]["mlp"]["expert"].update(ff=0),
    lambda d: d.update(width=0), lambda d: d.update(layers=[]),
])
def test_config_refuses_what_it_cannot_mean(change):
    d = json.loads(json.dumps({"architecture": "Nufusun", **NM.MODELS["mixed"][0]}))
    change(d)
    with pytest.raises(ValueError):
        NufusunConfig.from_dict(d)


def test_registry_and_checkpoint_roundtrip(tmp_path):
    cfg, w = NM.model("mixed")
    (tmp_path / "config.json").write_text(json.dumps(cfg.raw))
    save_file(w, tmp_path / "model.safetensors")
    c = load_config(tmp_path)
    assert of_config(c).name == "Nufusun" and c.layers == cfg.layers and c.path == str(tmp_path)
    got = c.load_weights()
    assert set(got) == set(w) and all(torch.equal(got[k], w[k]) for k in w)
    assert from_spec(json.loads(json.dumps(to_spec(c)))) == c  # what a replica process gets
    from kgs.serve.nufusun import NufusunModel

    assert of_config(c).serving_class() is NufusunModel and not NufusunModel.has_state


def test_checkpoint_shapes_are_checked():
    cfg, _ = NM.model("mixed")
    w = NM.weights(cfg, 12)  # any rows of the distance tables are fine below bias_max
    check_weights(cfg, w)
    for name in ("l0.mix.talk", "l0.mix.rel", "l0.mix.v.b", "l2.mlp.e6.down", "l3.mlp.router", "head"):
        bad = dict(w)
        bad[name] = w[name][..., :-1]
        with pytest.raises(ValueError, match=name.replace(".", r"\.")):
            check_weights(cfg, bad)
    with pytest.raises(ValueError, match="bias_max"):
        check_weights(cfg, NM.weights(cfg, 40))
    del w["final.norm"]
    with pytest.raises(ValueError, match="final.norm"):
        check_weights(cfg, w)
    assert "l1.mlp.router" not in tensor_shapes(cfg) and "l3.mlp.e2.up" in tensor_shapes(cfg)


# ------------------------------------------------------------------ distances
@pytest.mark.parametrize("rows,far", [(24, 200), (32, 128), (8, 20), (16, 100.5), (2, 5), (6, 10), (64, 1000)])
def test_buckets(rows, far):
    n = math.ceil(far) + 50
    b, half = buckets(rows, far, n), rows // 2
    assert b.tolist() == [O.bucket(i, rows, far) for i in range(n)]
    assert b[:half].tolist() == list(range(half)) and (np.diff(b) >= 0).all()
    assert b.max() == rows - 1 and (b[math.ceil(far):] == rows - 1).all()


def test_buckets_start_exactly():
    """Powers of a whole ratio: 16, 32, 64, 128, 256 begin a bucket each."""
    b = buckets(32, 256, 300)
    for k, n in enumerate((16, 32, 64, 128)):
        assert b[n] == 16 + 4 * k and b[n - 1] == 15 + 4 * k
    assert b[256] == b[255] == 31


def test_distance_table_is_mixed_and_ends_at_the_last_bucket():
    h = heads_of(6, 2, 16, 16, torch.float32)
    g = torch.Generator().manual_seed(0)
    talk, rel, temp = (torch.randn(s, generator=g) for s in ((6, 6), (10, 6), (6,)))
    t = TalkingWeights(h, talk, temp, rel, 0.3, 40, "cpu")
    for n in (0, 4, 5, 9, 39, 40, 400):
        want = talk.double() @ rel.double()[O.bucket(n, 10, 40)] / math.log(2)
        assert torch.allclose(t.bias[min(n, t.nfar), :6].double(), want, atol=1e-5)
    assert torch.allclose(t.sc.double(), temp.double() * 0.3 / math.log(2), atol=1e-6)


# ------------------------------------------------------------------- layouts
def _positions(chunk, lane):
    q = lane >> 4
    return [32 * chunk + 16 * (e // 4) + 4 * q + e % 4 for e in range(8)]


@pytest.mark.parametrize("heads,kv", [(6, 2), (5, 1), (32, 8), (20, 4), (8, 8)])
def test_mix_fragments(heads, kv):
    h = heads_of(heads, kv, 64, 64, torch.bfloat16)
    order = h.slot_heads()
    assert sorted(x for x in order if x >= 0) == list(range(heads)) and len(order) % 16 == 0
    for s in range(h.slots):  # heads of a slot share a key head
        assert len({x // h.group for x in order[4 * s:4 * s + 4] if x >= 0}) == 1
    t = torch.arange(heads * heads, dtype=torch.float64).reshape(heads, heads) + 1
    f = mix_fragments(t, order)
    for tile in range(f.shape[0]):
        for c in range(f.shape[1]):
            for lane in range(64):
                o = order[16 * tile + (lane & 15)]
                for e, p in enumerate(_positions(c, lane)):
                    g = order[p] if p < len(order) else -1
                    assert f[tile, c, lane, e] == (t[o, g] if o >= 0 and g >= 0 else 0)


def test_head_forms():
    bf = torch.bfloat16
    assert heads_of(32, 8, 128, 100, bf).tiled and heads_of(32, 8, 128, 100, bf).dvp == 128
    assert heads_of(18, 18, 32, 32, bf).mfma and not heads_of(18, 18, 32, 32, bf).tiled
    assert not heads_of(65, 5, 32, 32, bf).mfma and not heads_of(4, 2, 160, 32, bf).mfma
    assert heads_of(4, 2, 160, 40, bf).dkp == 160 and not heads_of(4, 2, 32, 32, torch.float32).mfma


# ---------------------------------------------------------------------- plans
def _plan(heads, n, pos0):
    from kgs.serve.nufusun import Geometry
    from kgs.serve.ragged import HostPack

    n, pos0 = np.array(n), np.array(pos0)
    row0 = np.cumsum(n) - n
    row_seq = np.repeat(np.arange(len(n)), n)
    pos = pos0[row_seq] + np.arange(n.sum()) - row0[row_seq]
    bt = np.arange(len(n) * 40).reshape(len(n), 40)
    pk = HostPack(torch.device("cpu"))
    refs = [pk.add(a) for a in (pos, pos, row_seq, row0, n, pos0, pos0, bt, pos, pos)]
    build = Geometry(heads).host_plan(pk, row0, n, pos0, bt, row_seq, pos, refs)
    return build(pk.send()), row0


def test_plan_splits_tiles_and_rows():
    h = heads_of(6, 3, 64, 64, torch.bfloat16)
    p, row0 = _plan(h, [1, 40, 2, 16, 15], [70, 3, 9, 500, 0])
    items = sorted(p.tiles.items.tolist())
    assert items == [[1, 1, 3, 32, 0, 2, -1, 0], [33, 1, 35, 8, 0, 2, -1, 0], [43, 3, 500, 16, 0, 17 // 2, 0, 0],
                     [43, 3, 500, 16, 8, 17, 1, 0]]
    pages = [i[5] - i[4] for i in p.tiles.items.tolist()]
    assert pages == sorted(pages, reverse=True)
    assert p.tiles.merges.tolist() == [[43, 16, 0, 2]] and p.tiles.parts == 2
    assert p.rows.n == 18 and p.rows.rows.tolist() == [0, 41, 42, *range(59, 74)]
    assert p.rows.tok_seq.tolist() == [0, 2, 2] + [4] * 15 and p.rows.tok_pos.tolist() == [70, 9, 10, *range(15)]
    p, _ = _plan(heads_of(32, 8, 64, 64, torch.bfloat16), [40], [3])  # eight slots: tiles of 16
    assert sorted(p.tiles.items.tolist()) == [[0, 0, 3, 16, 0, 1, -1, 0], [16, 0, 19, 16, 0, 2, -1, 0], [32, 0, 35, 8, 0, 2, -1, 0]]
    assert p.tiles.merges is None
    p, _ = _plan(h, [1, 1], [5, 900])
    assert p.tiles is None and p.rows.rows is None and p.rows.tok_pos.tolist() == [5, 900]
    p, _ = _plan(h, [64], [0])
    assert p.rows is None
    p, _ = _plan(heads_of(18, 18, 64, 64, torch.bfloat16), [64], [0])  # no tiled kernel for it
    assert p.tiles is None and p.rows.n == 64


def test_tile_items_cover_every_page_once():
    for portions in ([(0, 0, 0, 8192)], [(0, 0, 33000, 700)], [(i * 700, i, 50 * i, 700) for i in range(9)], [(5, 2, 9000, 17)], [(0, 0, 0, 3)]):
        for tile in (16, 32):
            items, merges = tile_items(portions, tile)
            seen, parts = {}, {}
            for r, s, p, n, a, b, part, _ in items.tolist():
                assert 0 <= a < b <= (p + n - 1) // 32 + 1 and 0 < n <= tile
                seen.setdefault((r, s, p, n), []).append((a, b))
                if part >= 0:
                    parts.setdefault(r, []).append(part)
            for (r, s, p, n), v in seen.items():
                v.sort()
                assert v[0][0] == 0 and v[-1][1] == (p + n - 1) // 32 + 1 and all(x[1] == y[0] for x, y in zip(v, v[1:]))
                assert (len(v) > 1) == (r in parts)
            assert sorted(x for v in parts.values() for x in v) == list(range(sum(map(len, parts.values()))))
            assert {m[0]: (m[2], m[3]) for m in merges.tolist()} == {r: (min(v), len(v)) for r, v in parts.items()}
            assert sum(k[3] for k in seen) == sum(x[3] for x in portions) and (merges[:, 3] <= 64).all()
    items, _ = tile_items([(0, 0, 0, 8192)], 32)
    assert (items[:, 5] - items[:, 4]).max() <= 155


# --------------------------------------------------------------------- oracle
def test_oracle_mechanisms():
    """Each mechanism against its definition written out."""
    g = torch.Generator().manual_seed(3)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)  # noqa: E731
    x, w = r(3, 8), r(8)
    assert torch.allclose(O.rms_norm(x, w, 0.5)[1, 2], x[1, 2] / ((x[1] ** 2).mean() + 0.5).sqrt() * (1 + w[2]))
    q, k = r(4, 6, 5), r(4, 2, 5)
    s = O.scores(q, k, 0.3, torch.arange(6.0, dtype=torch.float64))
    assert torch.allclose(s[2, 1, 4], (q[2, 4] * k[1, 1]).sum() * 0.3 * 4)
    t = r(6, 6)
    assert torch.allclose(O.talk(s, t)[2, 1, 5], sum(t[5, h] * s[2, 1, h] for h in range(6)))
    p = O.softmax_plus_one(s)
    e = torch.exp(s[2, :3, 1])
    assert torch.allclose(p[2, :3, 1], e / (1 + e.sum())) and p[2, 3, 1] == 0
    rel = r(8, 6)
    b = O.distance_bias(rel, 20, 30)
    assert torch.equal(b[25, 24], rel[1]) and torch.equal(b[25, 5], rel[7]) and torch.equal(b[25, 19], rel[O.bucket(6, 8, 20)])
    h, gate, up, down = r(8), 5 * r(12, 8), 5 * r(12, 8), r(8, 12)
    a, u = torch.clamp(gate @ h, max=0.7), torch.clamp(up @ h, -0.7, 0.7)
    assert a.min() < -0.7 and torch.allclose(O.expert(h, gate, up, down, 0.7), down @ (a / (1 + torch.exp(-1.702 * a)) * (u + 1)))
    idx, wt = O.route(r(5, 8), r(9, 8), 3)
    assert idx.shape == (5, 3) and ((wt > 0) & (wt < 1)).all() and (wt[:, :-1] >= wt[:, 1:]).all()
