"""Ruruzen without a GPU: configuration and checkpoint reading, the registry, the
scheduler's state slots and fed sequences, launch plans, and the oracle itself."""
import json
import os
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import hybrid_models as HM  # noqa: E402
from oracles import ruruzen as O  # noqa: E402

from kgs.models.registry import from_spec, load_config, of_config, to_spec  # noqa: E402
from kgs.models.ruruzen import RuruzenConfig, check_weights, tensor_shapes  # noqa: E402
from kgs.utils.safetensors import load_file, save_file  # noqa: E402


# ------------------------------------------------------------ configuration
def test_config_reads_every_size():
    c = HM.config("odd")
    assert (c.vocab, c.width, c.streams, c.eps, c.logit_softcap) == (203, 140, 3, 3e-6, 12.5)
    assert [x.type for x in c.layers] == ["channel_delta", "latent_attention", "channel_delta", "latent_attention",
                                          "latent_attention"]
    m = c.layers[3].mixer
    assert (m.heads, m.dim, m.vdim, m.q_rank, m.kv_rank, m.scale, m.kv_from) == (3, 56, 16, 20, 72, 0.09, 1)
    d = c.layers[0].mixer
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.conv, c.layers[0].ff, c.layers[2].ff) == (6, 2, 20, 28, 3, 90, None)
    assert c.has_state and not HM.config("attention").has_state


@pytest.mark.parametrize("change", [
    lambda d: d.update(architecture="Llama"),
    lambda d: d["layers"][3]["mixer"].update(kv_from=4),   # a later layer
    lambda d: d["layers"][3]["mixer"].update(kv_from=0),   # a layer without a latent
    lambda d: d["layers"][4]["mixer"].update(kv_from=3),   # a layer that reads another's
    lambda d: d["layers"][3]["mixer"].update(kv_rank=71),  # other latent size
    lambda d: d["layers"][0]["mixer"].update(kv_heads=4),  # heads not a multiple
    lambda d: d["layers"][0]["mlp"].update(kind="moe"),
    lambda d: d["layers"][0].update(type="window"),
    lambda d: d.update(width=0),
])
def test_config_refuses_what_it_cannot_mean(change):
    d = json.loads(json.dumps({"architecture": "Ruruzen", **HM.MODELS["odd"]}))
    change(d)
    with pytest.raises(ValueError):
        RuruzenConfig.from_dict(d)


def test_registry_and_checkpoint_roundtrip(tmp_path):
    raw = {"architecture": "Ruruzen", **HM.MODELS["odd"]}
    cfg = HM.config("odd")
    w = HM.weights(cfg, gate_rank=12)
    (tmp_path / "config.json").write_text(json.dumps(raw))
    save_file(w, tmp_path / "model.safetensors")
    c = load_config(tmp_path)
    assert of_config(c).name == "Ruruzen" and c.layers == cfg.layers and c.path == str(tmp_path)
    got = c.load_weights()
    assert set(got) == set(w) and all(torch.equal(got[k], w[k]) for k in w)
    again = from_spec(json.loads(json.dumps(to_spec(c))))  # what a replica process gets
    assert again == c
    from kgs.models.llama import LlamaConfig

    mc = LlamaConfig(hidden=256, heads=2, kv_heads=1)
    assert from_spec(to_spec(mc)) == mc
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Other"}))
    with pytest.raises(ValueError, match="Other"):
        load_config(tmp_path)


def test_checkpoint_shapes_are_checked():
    cfg = HM.config("odd")
    w = HM.weights(cfg, gate_rank=7)  # any rank of the low-rank gates is fine
    check_weights(cfg, w)
    for name in ("l1.mix.uk", "l0.mix.q.conv", "l0.mix.a2", "l2.hc1.mix", "embed"):
        bad = dict(w)
        bad[name] = w[name][..., :-1]
        with pytest.raises(ValueError, match=name.replace(".", r"\.")):
            check_weights(cfg, bad)
    del w["final.norm"]
    with pytest.raises(ValueError, match="final.norm"):
        check_weights(cfg, w)
    assert "l3.mix.dkv" not in tensor_shapes(cfg) and "l1.mix.dkv" in tensor_shapes(cfg)
    assert "l2.norm2" not in tensor_shapes(cfg) and "l2.hc2.in" not in tensor_shapes(cfg)


def test_safetensors_refuses_broken_files(tmp_path):
    p = tmp_path / "x.safetensors"
    save_file({"a": torch.arange(6, dtype=torch.int32).reshape(2, 3), "b": torch.ones(3, dtype=torch.bfloat16)}, p)
    t = load_file(p)
    assert t["a"].tolist() == [[0, 1, 2], [3, 4, 5]] and t["b"].dtype == torch.bfloat16
    raw = p.read_bytes()
    for broken in (raw[:-1], raw[:4], b"\xff" * 8 + raw[8:]):
        p.write_bytes(broken)
        with pytest.raises(ValueError):
            load_file(p)


# ----------------------------------------------------------------- scheduler
def _sched(**kw):
    from kgs._native import _serve

    c = _serve.SchedulerConfig()
    c.num_pages, c.max_batch, c.max_model_len, c.pad_multiple, c.state_slots = 20, 4, 512, 1, 4
    for k, v in kw.items():
        setattr(c, k, v)
    return _serve.Scheduler(c)


def test_fed_sequences_mix_portions_and_single_tokens():
    s = _sched()
    assert s.open(1) and s.open(2) and not s.open(1)
    p = s.feed([1, 2], [np.arange(40, dtype=np.int32), [5]])  # a first token is a portion too
    assert (p.kind, p.n_prefill, p.seq_lens.tolist(), p.ctx_starts.tolist()) == (3, 2, [40, 1], [0, 0])
    slots = dict(zip(p.seq_ids.tolist(), p.state_slots.tolist()))
    assert len(set(slots.values())) == 2 and 0 not in slots.values()
    p = s.feed([2, 1], [[7], [1, 2]])
    assert (p.kind, p.seq_ids.tolist(), p.n_prefill) == (3, [1, 2], 1)
    assert p.positions.tolist() == [40, 41, 1] and p.ctx_lens.tolist() == [2]
    assert [slots[i] for i in p.seq_ids.tolist()] == p.state_slots.tolist()
    p = s.feed([2], [[8]])
    assert p.kind == 2 and p.positions.tolist() == [2] and s.check_invariants() == ""
    # refused whole, nothing changed: unknown id, twice the same, no tokens, too many pages
    free = s.num_free_pages
    for ids, toks in (([3], [[1]]), ([1, 1], [[1], [2]]), ([1], [[]]), ([1], [np.zeros(500, np.int32)]),
                      ([1, 2], [np.zeros(460, np.int32), np.zeros(400, np.int32)])):
        assert s.feed(ids, toks).kind == 0
    assert s.num_free_pages == free and s.info(1)["cached"] == 42
    assert s.abort(1) and s.abort(2)
    assert s.num_free_pages == 19 and s.check_invariants() == ""


def test_fed_and_generated_sequences_share_pages_and_slots():
    s = _sched(state_slots=2, max_batch=2)
    assert s.open(10)
    s.add(1, np.arange(5, dtype=np.int32), 4)
    s.add(2, np.arange(6, dtype=np.int32), 4)
    p = s.schedule()
    assert p.kind == 1 and p.seq_ids.tolist() == [1] and p.pf_block_tables.shape == (1, 1)  # one slot left
    assert not s.open(11)
    s.update(p.seq_ids, np.array([3], np.int32), np.array([1], np.uint8))  # 1 stops: its slot is free
    p2 = s.schedule()
    assert p2.seq_ids.tolist() == [2] and p2.state_slots.tolist() == p.state_slots.tolist()
    assert s.check_invariants() == ""


@pytest.mark.parametrize("chunk", [0, 40])
def test_state_slots_follow_random_traffic(chunk):
    """Admissions, stops and preemptions: every running sequence has its own slot."""
    rng = np.random.default_rng(chunk)
    s = _sched(num_pages=9, chunk_tokens=chunk, max_model_len=200)
    for i in range(12):
        s.add(i, rng.integers(0, 9, size=int(rng.integers(1, 70))).astype(np.int32), int(rng.integers(1, 40)))
    preempted = 0
    for _ in range(600):
        p = s.schedule()
        if p.kind == 0:
            break
        preempted += len(p.preempted)
        assert len(p.state_slots) == len(p.seq_ids) == len(set(p.state_slots.tolist()))
        assert p.state_slots.min() >= 1 and s.check_invariants() == ""
        ids = p.seq_ids
        if p.kind == 3:
            ids = np.concatenate([ids[:p.n_prefill][p.last_chunk.astype(bool)], ids[p.n_prefill:]])
        s.update(ids, np.ones(len(ids), np.int32), np.zeros(len(ids), np.uint8))
    assert s.num_running == s.num_waiting == 0 and preempted > 0 and s.num_free_pages == 8


# --------------------------------------------------------------------- plans
def test_launch_plan_splits_portions_and_orders_rows():
    from kgs.serve.hybrid import Geometry, HostPack

    g = Geometry(heads=4, rp=256, hd=64)
    # behind a long context a portion is worth expanding from rp hd / (rp - hd) = 85 tokens on, at the start from 16
    assert g.expand(86, 10 ** 6) and not g.expand(85, 10 ** 6) and g.expand(16, 0) and not g.expand(15, 0)
    assert not Geometry(4, 64, 64).expand(10000, 0) and not Geometry(4, 256, 0).expand(999, 0)
    n = np.array([300, 3, 130, 1])
    pos0 = np.array([0, 31, 64, 99])
    row0 = np.cumsum(n) - n
    bt = np.arange(4 * 20).reshape(4, 20)
    row_seq = np.repeat(np.arange(4), n)
    pos = pos0[row_seq] + np.arange(n.sum()) - row0[row_seq]
    pk = HostPack(torch.device("cpu"))
    refs = [None] * 9
    (r, shape), e = g.lay_out(pk, row0, n, pos0, bt, row_seq, pos, refs)
    get = pk.send()
    assert shape["nt"] == 4 and get(r["rows"]).tolist() == [300, 301, 302, 433]
    assert get(r["q0"]).tolist() == [0, 3] and get(r["n"]).tolist() == [3, 1]
    assert get(r["tok_pos"]).tolist() == [31, 32, 33, 99] and get(r["tok_seq"]).tolist() == [0, 0, 0, 1]
    assert get(r["items"]).tolist() == [[1, 0], [0, 0]] and get(r["bt"]).tolist() == bt[[1, 3]].tolist()
    items, ctx = get(e[0]), get(e[1])
    assert len(ctx) == 300 + 194 and ctx[300 + 33].item() == bt[2][1] * 32 + 1
    assert sorted(items.tolist()) == [[0, 0, 0, 128], [128, 0, 128, 128], [256, 0, 256, 44], [303, 300, 64, 128],
                                      [431, 300, 192, 2]]
    ends = (items[:, 2] + items[:, 3]).tolist()
    assert ends == sorted(ends, reverse=True)


def test_delta_chunk_plan():
    from kgs.ops.delta import chunk_plan

    n = np.array([3, 40, 1, 16])
    row0 = np.array([0, 3, 43, 44])
    pos0, slot = np.array([5, 6, 7, 0]), np.array([4, 3, 2, 1])
    p = chunk_plan(row0, n, pos0, slot)
    assert p["chunks"].tolist() == [[3, 16, 1, 0, 3, 6, 3, 0], [19, 16, 1, 0, 3, 6, 3, 0], [35, 8, 1, 0, 3, 6, 3, 0],
                                    [44, 16, 3, 0, 44, 0, 1, 0]]
    assert p["cseqs"].tolist() == [[1, 0, 3, 3], [3, 3, 1, 44]]
    assert p["step_rows"].tolist() == [0, 1, 2, 43] and p["step_seqs"].tolist() == [0, 2]
    assert chunk_plan(row0[:1], n[:1], pos0[:1], slot[:1]) == {}


# -------------------------------------------------------------------- oracle
def test_oracle_delta_rule_by_hand():
    """One head, one key channel: the recurrence in scalars."""
    q, k, v = torch.tensor([2.0, 3.0]), torch.tensor([1.0, 0.5]), torch.tensor([4.0, 6.0])
    g, beta = torch.tensor([0.9, 0.5]), torch.tensor([0.25, 0.5])
    s1 = 0.25 * 4.0
    s2 = 0.5 * s1 + 0.5 * (0.5 * (6.0 - 0.5 * s1 * 0.5))
    o, s = O.delta_rule(q[:, None, None], k[:, None, None], v[:, None, None], g[:, None, None], beta[:, None])
    assert torch.allclose(o.flatten(), torch.tensor([2 * s1, 3 * s2])) and abs(s.item() - s2) < 1e-6


def test_oracle_planted_mistakes_show():
    """Each mistake in the oracle moves the logits by far more than rounding: the
    test models are sensitive to what the GPU tests check."""
    tokens = np.random.default_rng(0).integers(0, 203, size=40).tolist()
    cfg = HM.config("odd")
    raw, w = cfg.raw, {k: v.double() for k, v in HM.weights(cfg).items()}
    base = O.forward(raw, w, tokens)

    def moved(other):
        return float((other - base).pow(2).mean().sqrt() / base.std())

    def run(patch=None, weights=None, config=None):
        saved = {n: getattr(O, n) for n in patch or {}}
        try:
            for n, f in (patch or {}).items():
                setattr(O, n, f)
            return moved(O.forward(config or raw, weights or w, tokens))
        finally:
            for n, f in saved.items():
                setattr(O, n, f)

    hyper_out, conv, delta, attn = O.hyper_out, O.short_conv, O.delta_rule, O.causal_softmax_attention
    assert run() == 0
    assert run({"hyper_out": lambda x, y, m, o: hyper_out(x, y, m.T, o)}) > 1e-3       # mix is [from, to]
    assert run({"short_conv": lambda x, c: conv(x, c.flip(1))}) > 1e-2
    assert run({"delta_rule": lambda q, k, v, g, b: delta(q, k, v, g.mean(-1, keepdim=True).expand_as(g), b)}) > 1e-3
    assert run({"causal_softmax_attention":
                lambda q, k, v, s: attn(q[:, :, :], torch.cat([k[1:], k[:1]]), v, s)}) > 1e-2
    assert run(weights={**w, "l3.mix.g": 0 * w["l3.mix.g"]}) > 1e-3
    shared = json.loads(json.dumps(raw))
    shared["layers"][3]["mixer"]["scale"] *= 1.5
    assert run(config=shared) > 1e-3
