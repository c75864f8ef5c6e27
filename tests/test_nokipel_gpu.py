"""Nokipel through the serving engine on the GPU: small models of other sizes than each
other, against the plain oracle -- whole prompts, token by token, portions, mixed
batches, pages and state slots used again, keys at chunk edges, long decoding, generation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import nokipel_models as NM  # noqa: E402
from oracles import nokipel as O  # noqa: E402

pytestmark = pytest.mark.gpu

# (median row, every row): rms over the vocabulary, against the logits' own. In bf16 a
# row where two experts nearly tie may choose the other one, which later rows then see:
# one in five (or one) may be further off.
TOL = {"float32": (3e-6, 2e-5), "bfloat16": (1.2e-2, 4e-2)}
NAMES = sorted(NM.MODELS)


def tokens(name, n, seed=0):
    return np.random.default_rng(seed).integers(0, NM.config(name).vocab, size=n).tolist()


def engine_of(cfg, w, dtype, pages, **kw):
    from kgs.serve import EngineConfig, LLMEngine

    object.__setattr__(cfg, "load_weights", lambda seed=0, device="cpu": w)
    return LLMEngine(cfg, EngineConfig(num_pages=pages, dtype=dtype, **{"max_batch": 4, "max_model_len": 1024, **kw}))


def engine(name, dtype="float32", pages=40, **kw):
    return engine_of(*NM.model(name), dtype, pages, **kw)


def row_errors(got, want):
    got, want = got.detach().cpu().double(), want.double()
    assert got.shape == want.shape
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.std()


def check(got, want, dtype, what=""):
    err = row_errors(got, want)
    mid, worst = TOL[dtype]
    off = torch.nonzero(~(err < worst))[:, 0].tolist()
    assert len(off) <= (0 if dtype == "float32" else max(1, len(err) // 5)), \
        f"{what}: rows {off[:9]} off by up to {float(err.max()):.2e}"
    assert dtype == "float32" or float(err.max()) < 0.8, f"{what}: row {int(err.argmax())} off by {float(err.max()):.2e}"
    assert len(err) < 8 or float(err.median()) < mid, f"{what}: median {float(err.median()):.2e}"


def feed_all(eng, toks, cuts):
    """One request in portions of these sizes; logits of every position."""
    rid, at, out = eng.open_feed(), 0, []
    for n in cuts:
        out.append(eng.feed([(rid, toks[at:at + n], list(range(n)))]))
        at += n
    assert at == len(toks)
    eng.close_feed(rid)
    assert eng.sched.check_invariants() == ""
    return torch.cat(out)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_whole_decode_and_portions(name, dtype):
    """Every way to cut a prompt gives the oracle's logits at every position."""
    T = 110
    toks = tokens(name, T)
    want = NM.oracle_logits(name, toks)
    eng = engine(name, dtype)
    for cuts in ([T], [1] * T, [2] * 20 + [70], [31, 1, 32, 1, 2, 43], [3, 61, 2, 44], [63, 2, 45], [97, 13], [16, 15, 17, 62]):
        check(feed_all(eng, toks, cuts), want, dtype, f"{name} {cuts[:6]}")
    assert eng.stats["graph_replays"] > 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_residual_after_every_layer_run(name, dtype):
    cfg, w = NM.model(name)
    toks = tokens(name, 37, seed=2)
    ref, got = [], []
    O.forward(cfg.raw, w, toks, layers=ref)
    eng = engine(name, dtype)
    eng.model.on_layer = lambda i, x: got.append((i, x.clone()))
    feed_all(eng, toks, [37])
    assert [i for i, _ in got] == list(range(len(cfg.runs)))
    for (i, x), r in zip(got, ref):
        err = ((x.cpu().double() - r).pow(2).mean(-1).sqrt() / r.pow(2).mean(-1).sqrt()).median()
        assert err < (2e-6 if dtype == "float32" else 2e-2), (i, float(err))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_unequal_requests_in_one_batch(name, dtype):
    """Portions beside single tokens, a request that waits, one that ends and one
    that takes over its pages: each as if alone."""
    eng = engine(name, dtype, pages=15)  # 14 pages of 32: the requests together need more
    lens = {"a": 130, "b": 66, "c": 95, "d": 120, "e": 40}
    toks = {k: tokens(name, n, seed=ord(k)) for k, n in lens.items()}
    at, ids, out = dict.fromkeys(lens, 0), {}, {k: [] for k in lens}
    steps = [dict(a=64, b=2, c=1), dict(a=1, b=30, c=31), dict(b=1, c=2), dict(a=2, b=1, c=1, d=33), dict(a=1, b=1, c=1, d=1),
             dict(c=59, d=3, b=31), dict(a=33, e=1), dict(a=29, d=1, e=2), dict(d=80, e=33), dict(e=3, d=1),
             dict(e=1, d=1)]
    for st in steps:
        entries = []
        for k, n in st.items():
            if k not in ids:
                ids[k] = eng.open_feed()
            entries.append((ids[k], toks[k][at[k]:at[k] + n], list(range(n))))
        lg, r = eng.feed(entries), 0
        for k, n in st.items():
            out[k].append(lg[r:r + n])
            r += n
            at[k] += n
            if at[k] == lens[k]:
                eng.close_feed(ids[k])
        assert eng.sched.check_invariants() == ""
    assert at == lens
    for k in lens:
        check(torch.cat(out[k]), NM.oracle_logits(name, toks[k]), dtype, k)


def test_a_batch_changes_nothing():
    """The same request alone and beside others, on other pages."""
    name = "mixed"
    toks = tokens(name, 80)
    for dtype in ("float32", "bfloat16"):
        eng = engine(name, dtype)
        alone = feed_all(eng, toks, [50, 28, 1, 1])
        others = [eng.open_feed() for _ in range(2)]
        eng.feed([(others[0], tokens(name, 45, 5), []), (others[1], tokens(name, 3, 6), [])])
        eng.close_feed(others.pop(0))
        rid, got, at = eng.open_feed(), [], 0
        for n in (50, 28, 1, 1):
            got.append(eng.feed([(others[0], tokens(name, 1 + n % 3, n), []),
                                 (rid, toks[at:at + n], list(range(n)))]))
            at += n
        err = row_errors(torch.cat(got), alone.double().cpu())
        assert float(err.median()) < (1e-6 if dtype == "float32" else 1e-2)


def _pointer_model(chunk):
    """One attention layer that finds token 1 from token 0 by a score that stands out."""
    raw = {"architecture": "Nokipel", "vocab": 8, "width": 64, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5, "groups": 2},
           "layers": [NM.attention(3, 1, 64, 64, 0.125, chunk, (2, 10.0), NM.dense(32, 1.0)),
                      NM.attention(2, 2, 32, 16, 0.2, 1, (8, 50.0))]}
    from kgs.models.nokipel import NokipelConfig

    cfg = NokipelConfig.from_dict(raw)
    w = NM.weights(cfg, seed=3)
    g = torch.Generator().manual_seed(1)
    turn = torch.linalg.qr(torch.randn(64, 64, generator=g))[0]
    m = "l0.mix."
    w[m + "q"] = torch.cat([torch.eye(64)] * 3).to(torch.bfloat16)
    w[m + "k"], w[m + "v"] = turn.to(torch.bfloat16), torch.eye(64, dtype=torch.bfloat16)
    for n in ("q.b", "k.b", "v.b"):
        w[m + n] = w[m + n] * 0
    w["l0.norm1"] = w["l0.norm1"] * 0 + 1.5
    w[m + "o"] = torch.cat([torch.eye(64)] * 3, 1).to(torch.bfloat16)
    e = torch.randn(8, 64, generator=g)
    e[1] = turn.T @ e[0]        # token 1's key is what token 0 asks for
    w["embed"] = e.to(torch.bfloat16)
    return cfg, w


T_FAR = 131


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("chunk,far", [(500, 0), (500, 1), (500, 31), (500, 64), (500, 129), (100, 100), (100, 99), (100, 101),
                                       (128, 128), (128, 127), (130, 130), (65, 65), (65, 64), (33, 99), (33, 98), (1, 129)])
def test_keys_at_chunk_edges_in_prompt_and_decode(dtype, chunk, far):
    """The last query's best key stands far back, at page borders, just inside or just
    outside its chunk: a key lost, shifted or let in changes the logits."""
    cfg, w = _pointer_model(chunk)
    toks = np.random.default_rng(far).integers(2, 8, size=T_FAR).tolist()
    toks[far], toks[T_FAR - 1] = 1, 0
    want = O.forward(cfg.raw, w, toks)
    without = list(toks)
    without[far] = 2
    gap = float((O.forward(cfg.raw, w, without)[-1] - want[-1]).pow(2).mean().sqrt() / want.std())
    inside = far // chunk == (T_FAR - 1) // chunk
    if far != T_FAR - 1:
        assert (gap > 0.1) if inside else gap == 0, gap  # the far key decides the last logits, or no logit
    if not inside:  # how far off the logits were if it were seen
        mask, O.chunk_mask = O.chunk_mask, lambda T, s: torch.ones(T, T, dtype=torch.bool).tril() if s == chunk else mask(T, s)
        gap = float((O.forward(cfg.raw, w, toks)[-1] - want[-1]).pow(2).mean().sqrt() / want.std())
        O.chunk_mask = mask
        assert gap > 0.05, gap
    eng = engine_of(cfg, w, dtype, 12, max_batch=2, max_model_len=256)
    for cuts in ([T_FAR], [T_FAR - 1, 1], [T_FAR - 2, 2], [far + 1, T_FAR - far - 1] if far + 1 < T_FAR else [T_FAR], [64, 66, 1]):
        err = row_errors(feed_all(eng, toks, cuts), want)
        assert float(err[-1]) < (1e-4 if dtype == "float32" else 0.25 * max(gap, 0.1)), (far, cuts, float(err[-1]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("far", [0, 15, 16, 63, 64, 100, 127])
def test_a_far_token_reaches_the_last_logits_through_the_state(dtype, far):
    """Lightning layers only, decays near 1: another token far back moves the last logits,
    however the sequence was cut; a state lost at a cut would not."""
    raw = {"architecture": "Nokipel", "vocab": 8, "width": 64, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5, "groups": 1},
           "layers": [NM.lightning(16, 24, [1.0, 0.9999], NM.dense(32, 1.0))]}
    from kgs.models.nokipel import NokipelConfig

    cfg = NokipelConfig.from_dict(raw)
    w = NM.weights(cfg, seed=5)
    u = torch.nn.functional.normalize(torch.randn(64, generator=torch.Generator().manual_seed(2)), dim=0)
    w["l0.mix.k"] = (2 * u).expand(32, 64).to(torch.bfloat16).contiguous()  # token 1 alone has a loud key
    w["embed"][1] = (8 * u).to(torch.bfloat16)
    T = 131
    toks = np.random.default_rng(far).integers(2, 8, size=T).tolist()
    want_without = O.forward(raw, w, toks)
    toks[far] = 1
    want = O.forward(raw, w, toks)
    gap = float((want_without[-1] - want[-1]).pow(2).mean().sqrt() / want.std())
    assert gap > 0.05, gap
    eng = engine_of(cfg, w, dtype, 12, max_batch=2, max_model_len=256)
    for cuts in ([T], [T - 1, 1], [T - 2, 2], [far + 1, T - far - 1], [64, 66, 1], [100] + [1] * 31, [2] * 65 + [1]):
        err = row_errors(feed_all(eng, toks, cuts), want)
        assert float(err[-1]) < (1e-4 if dtype == "float32" else 0.4 * gap), (far, cuts, float(err[-1]), gap)


def test_a_freed_state_slot_starts_from_zeros():
    """A request in a slot that another one left, whose first portion has one token, two,
    or a chunk: as in a fresh engine."""
    for dtype in ("float32", "bfloat16"):
        eng = engine("first", dtype, max_batch=1)
        for n in (1, 2, 40):
            feed_all(eng, tokens("first", 50, seed=n), [20, 30])
            toks = tokens("first", n + 5, seed=100 + n)
            check(feed_all(eng, toks, [n, 1, 4]), NM.oracle_logits("first", toks), dtype, f"{n} tokens first")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens(dtype):
    """Sequences of one to four tokens."""
    for name in NAMES:
        eng = engine(name, dtype)
        for n in (1, 2, 3, 4):
            toks = tokens(name, n, seed=40 + n)
            for cuts in ([n], [1] * n):
                check(feed_all(eng, toks, cuts), NM.oracle_logits(name, toks), dtype, f"{name} {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    """300 decoded tokens, over nine page borders and several graph widths."""
    toks = tokens("mixed", 320, seed=9)
    want = NM.oracle_logits("mixed", toks)
    check(feed_all(engine("mixed", dtype), toks, [20] + [1] * 300), want, dtype)


def test_graph_replays_equal_eager_steps():
    """Decode steps of changing batches: every replay gives what the same step gives
    without a graph, with prompts in between."""
    a, b = engine("first", "bfloat16"), engine("first", "bfloat16", cuda_graphs=False)
    rng = np.random.default_rng(0)
    ids = [[e.open_feed() for _ in range(4)] for e in (a, b)]
    for step in range(24):
        sel = rng.permutation(4)[:rng.integers(1, 5)]
        toks = {int(i): tokens("first", 20 if step % 7 == 0 else 1, seed=100 * step + int(i)) for i in sel}
        out = [e.feed([(x[i], t, [len(t) - 1]) for i, t in toks.items()]) for e, x in zip((a, b), ids)]
        assert float(row_errors(out[0], out[1].double().cpu()).max()) < 1e-6, step
    assert a.stats["graph_replays"] > 8 and b.stats["graph_replays"] == 0


def _greedy_ok(name, prompts, outs, dtype):
    for p, r in zip(prompts, outs):
        lg = NM.oracle_logits(name, list(p) + r.output)
        bad = [i for i, t in enumerate(r.output)
               if lg[len(p) - 1 + i][t] < lg[len(p) - 1 + i].max() - (1e-4 if dtype == "float32" else 0.3) * lg.std()]
        assert not bad if dtype == "float32" else len(bad) <= 1, (len(p), bad)


@pytest.mark.parametrize("kw", [dict(), dict(chunked_prefill=24), dict(overlap=False), dict(cuda_graphs=False),
                                dict(pages=9, max_model_len=200), dict(prefix_caching=True, chunked_prefill=64)],
                         ids=["plain", "chunked", "no-overlap", "eager", "preempt", "prefix"])
@pytest.mark.parametrize("name", ["mixed", "stateless"])
def test_greedy_generation(name, kw):
    """The engine's own entry point, scheduler and sampler."""
    from kgs.serve import SamplingParams

    if "prefix_caching" in kw and NM.config(name).has_state:
        with pytest.raises(ValueError, match="prefix caching"):
            engine(name, "float32", **kw)
        return
    eng = engine(name, "float32", **{"max_batch": 3, **kw})
    prompts = [tokens(name, n, seed=n) for n in (1, 33, 60, 7, 64)]
    if "prefix_caching" in kw:
        prompts += [prompts[4] + [5, 6, 7], prompts[4][:40] + [9]]
    outs = eng.generate(prompts, SamplingParams(max_tokens=45, ignore_eos=True))
    assert [len(r.output) for r in outs] == [45] * len(prompts)
    _greedy_ok(name, prompts, outs, "float32")
    if "pages" in kw:
        assert eng.stats["preemptions"] > 0
    assert eng.sched.check_invariants() == "" and eng.sched.num_running == 0


def test_greedy_generation_bf16_and_sampling():
    from kgs.serve import SamplingParams

    eng = engine("mixed", "bfloat16", chunked_prefill=40)
    prompts = [tokens("mixed", n, seed=n) for n in (5, 130, 70)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True))
    _greedy_ok("mixed", prompts, outs, "bfloat16")
    p = SamplingParams(max_tokens=6, temperature=0.9, top_k=20, top_p=0.9, seed=4, logprobs=2, ignore_eos=True)
    a, b = (eng.generate(prompts, p) for _ in range(2))
    assert [r.output for r in a] == [r.output for r in b] and all(len(r.logprobs) == 6 for r in a)


def test_pages_sized_from_memory():
    from kgs.serve import EngineConfig, LLMEngine

    cfg, w = NM.model("mixed")
    object.__setattr__(cfg, "load_weights", lambda seed=0, device="cpu": w)
    eng = LLMEngine(cfg, EngineConfig(max_batch=2, max_model_len=300))
    assert eng.num_pages == 2 * 10 + 1


def test_engine_refuses_what_the_model_has_not():
    for kw in (dict(kv_cache_dtype="fp8"), dict(decode_weights="fp8"), dict(prefill_weights="fp8")):
        with pytest.raises(ValueError):
            engine("mixed", **kw)
    eng = engine("mixed", pages=4)
    rid = eng.open_feed()
    with pytest.raises(RuntimeError, match="does not fit"):
        eng.feed([(rid, tokens("mixed", 200), [])])
    with pytest.raises(RuntimeError, match="tokens outside"):
        eng.feed([(rid, [203], [])])


def test_trace_run_program(tmp_path):
    """bin/trace_run as a program: steps on standard input, logits in files."""
    from kgs.utils.safetensors import save_file

    cfg, w = NM.model("mixed")
    (tmp_path / "config.json").write_text(json.dumps(cfg.raw))
    save_file(w, tmp_path / "model.safetensors")
    toks = {k: tokens("mixed", n, seed=n) for k, n in (("x", 40), ("y", 9))}
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks["x"][:30], "want": [0, 29]},
                                     {"id": "y", "tokens": toks["y"][:8], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks["x"][30:39], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "y", "tokens": toks["y"][8:], "want": [0]},
                                     {"id": "x", "tokens": toks["x"][39:], "want": [0]}], "end": ["x", "y"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "128"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    wx, wy = (NM.oracle_logits("mixed", toks[k]) for k in "xy")
    read = lambda n: torch.from_numpy(np.fromfile(tmp_path / f"{n}.f32", "<f4")).reshape(-1, cfg.vocab)  # noqa: E731
    check(read(0), wx[[0, 29]], "float32")
    check(read(2), torch.stack([wy[8], wx[39]]), "float32")
    assert not (tmp_path / "1.f32").exists()


def test_serving_benchmark_on_a_model_folder(tmp_path, capsys):
    """The command line, from a checkpoint to generated tokens."""
    from kgs.serve.bench import main
    from kgs.utils.safetensors import save_file

    cfg, w = NM.model("first")
    (tmp_path / "config.json").write_text(json.dumps(cfg.raw))
    save_file(w, tmp_path / "model.safetensors")
    assert main(["--model", str(tmp_path), "--requests", "5", "--input-len", "33", "--output-len", "6", "--max-batch", "4",
                 "--max-model-len", "256", "--chunked-prefill", "48"]) == 0
    out = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert out["output_tok_per_s"] > 0 and out["stats"]["decode_tokens"] >= 5 * 5
