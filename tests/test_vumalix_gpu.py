"""Vumalix through the serving engine on the GPU: small models of other sizes than each
other, against the plain oracle -- whole prompts, token by token, portions, mixed
batches, pages and state slots used again, keys at window edges and far back, the
convolutions' inputs across cuts, long decoding, generation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import vumalix_models as VM  # noqa: E402
from oracles import vumalix as O  # noqa: E402

pytestmark = pytest.mark.gpu

# (median row, every row): rms over the vocabulary, against the logits' own. In bf16 a row whose two
# maps nearly cancel loses more (rounding the oracle's projections alone moves one row by 4.6e-2)
TOL = {"float32": (5e-6, 3e-5), "bfloat16": (1.8e-2, 7e-2)}
NAMES = sorted(VM.MODELS)


def tokens(name, n, seed=0):
    return np.random.default_rng(seed).integers(0, VM.config(name).vocab, size=n).tolist()


def engine_of(cfg, w, dtype, pages, **kw):
    from kgs.serve import EngineConfig, LLMEngine

    object.__setattr__(cfg, "load_weights", lambda seed=0, device="cpu": w)
    return LLMEngine(cfg, EngineConfig(num_pages=pages, dtype=dtype, **{"max_batch": 4, "max_model_len": 1024, **kw}))


def engine(name, dtype="float32", pages=40, **kw):
    return engine_of(*VM.model(name), dtype, pages, **kw)


def row_errors(got, want):
    got, want = got.detach().cpu().double(), want.double()
    assert got.shape == want.shape
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.std()


def check(got, want, dtype, what=""):
    err = row_errors(got, want)
    mid, worst = TOL[dtype]
    assert float(err.max()) < worst, f"{what}: row {int(err.argmax())} off by {float(err.max()):.2e}"
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
    want = VM.oracle_logits(name, toks)
    eng = engine(name, dtype)
    for cuts in ([T], [1] * T, [2] * 20 + [70], [31, 1, 32, 1, 2, 43], [3, 61, 2, 44], [63, 2, 45], [97, 13], [16, 15, 17, 62]):
        check(feed_all(eng, toks, cuts), want, dtype, f"{name} {cuts[:6]}")
    assert eng.stats["graph_replays"] > 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_residual_after_every_layer(name, dtype):
    cfg, w = VM.model(name)
    toks = tokens(name, 37, seed=2)
    ref, got = [], []
    O.forward(cfg.raw, w, toks, layers=ref)
    eng = engine(name, dtype)
    eng.model.on_layer = lambda i, x: got.append((i, x.clone()))
    feed_all(eng, toks, [37])
    assert [i for i, _ in got] == list(range(len(cfg.layers)))
    for (i, x), r in zip(got, ref):
        err = ((x.cpu().double() - r).pow(2).mean(-1).sqrt() / r.pow(2).mean(-1).sqrt()).median()
        assert err < (5e-6 if dtype == "float32" else 2e-2), (i, float(err))


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
        check(torch.cat(out[k]), VM.oracle_logits(name, toks[k]), dtype, k)


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


def _pointer_model(kind, window=0, vocab=8):
    """One layer that finds token 1 from token 0 by a score that stands out."""
    from kgs.models.vumalix import VumalixConfig

    ff = 32
    layer = VM.latent(3, 64, 8, 64, 64, 64, window, 100.0, 0.125, ff) if kind == "latent" else \
        VM.attention(3, 1, 64, 64, 0.125, 0.4, (0.05, 50), ff)
    raw = {"architecture": "Vumalix", "vocab": vocab, "width": 64, "canon": {"taps": 3}, "norm": {"eps": 1e-5}, "layers": [layer]}
    cfg = VumalixConfig.from_dict(raw)
    w = VM.weights(cfg, seed=3)
    g = torch.Generator().manual_seed(1)
    turn = torch.linalg.qr(torch.randn(64, 64, generator=g))[0]
    m, eye = "l0.mix.", torch.eye(64)
    put = lambda n, t: w.__setitem__(n, t.to(torch.bfloat16))  # noqa: E731
    put("l0.canon1", 0.02 * torch.randn(64, 3, generator=g))
    if kind == "latent":
        put(m + "dq", eye)
        put(m + "uq", torch.cat([eye, 0.05 * torch.randn(8, 64, generator=g)]).repeat(3, 1))
        put(m + "dkv", torch.cat([eye, 0.05 * torch.randn(8, 64, generator=g)]))
        put(m + "uk", turn.repeat(3, 1))
        put(m + "uv", eye.repeat(3, 1))
        for n in ("dq.norm", "dkv.norm"):
            put(m + n, torch.ones(64))
    else:  # the second map looks at nothing in particular
        put(m + "q", torch.cat([eye, 0.05 * eye]).repeat(3, 1))
        put(m + "k", torch.cat([turn, 0.05 * torch.randn(64, 64, generator=g)]))
        put(m + "v", eye)
        for n in ("q.norm", "k.norm"):
            put(m + n, torch.ones(64))
    put(m + "o", torch.cat([eye] * 3, 1))
    put("l0.norm1", torch.tensor(2.0))
    e = torch.randn(vocab, 64, generator=g)
    e[1] = turn.T @ e[0]        # token 1's key is what token 0 asks for
    put("embed", e)
    return cfg, w


T_FAR = 131


def _far_key(kind, far, window, dtype):
    cfg, w = _pointer_model(kind, window or 1)
    toks = np.random.default_rng(far).integers(2, 8, size=T_FAR).tolist()
    toks[far], toks[T_FAR - 1] = 1, 0
    want = O.forward(cfg.raw, w, toks)

    def moved(**patch):
        """How far the last logits move: with the far token another one, or a patched oracle."""
        saved = {n: getattr(O, n) for n in patch}
        try:
            for n, f in patch.items():
                setattr(O, n, f)
            t = list(toks)
            if not patch:
                t[far] = 2
            return float((O.forward(cfg.raw, w, t)[-1] - want[-1]).pow(2).mean().sqrt() / want.std())
        finally:
            for n, f in saved.items():
                setattr(O, n, f)

    dist = T_FAR - 1 - far
    seen = not window or dist < window
    gap = moved()
    if dist > 2:  # else the convolution sees it too
        assert (gap > 0.1) if seen else gap < 0.02, gap
    if not seen:  # a window one key wider or narrower would show
        gap = moved(window_mask=lambda T, s, f=O.window_mask: f(T, max(s, dist + 1)))
        assert gap > 0.1, gap
    eng = engine_of(cfg, w, dtype, 12, max_batch=2, max_model_len=256)
    for cuts in ([T_FAR], [T_FAR - 1, 1], [T_FAR - 2, 2], [far + 1, T_FAR - far - 1] if far + 1 < T_FAR else [T_FAR], [64, 66, 1]):
        err = row_errors(feed_all(eng, toks, cuts), want)
        assert float(err[-1]) < (1e-4 if dtype == "float32" else 0.25 * max(gap, 0.1)), (far, cuts, float(err[-1]))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window,far", [(500, 0), (500, 1), (500, 64), (131, 0), (130, 0), (130, 1), (99, 32), (99, 31), (67, 64), (66, 64),
                                        (35, 96), (34, 96), (32, 98), (32, 99), (4, 127), (3, 127), (1, 125)])
def test_keys_at_window_edges_in_prompt_and_decode(dtype, window, far):
    """The last query's best key stands far back, at page borders, just inside or just
    outside its window: a key lost, shifted or let in changes the logits."""
    _far_key("latent", far, window, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("far", [0, 1, 31, 32, 63, 64, 97, 126])
def test_far_keys_of_differential_attention(dtype, far):
    _far_key("attention", far, 0, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("taps", [2, 3, 4, 6])
def test_the_convolution_reaches_over_every_cut(dtype, taps):
    """A loud token in front of a cut: the next taps - 1 positions see it through the state,
    and no later one. Nothing else carries it there (windows of one key)."""
    from kgs.models.vumalix import VumalixConfig

    raw = {"architecture": "Vumalix", "vocab": 8, "width": 64, "canon": {"taps": taps}, "norm": {"eps": 1e-5},
           "layers": [VM.latent(2, 32, 4, 32, 32, 32, 1, 10.0, 0.3, 32)]}
    cfg = VumalixConfig.from_dict(raw)
    w = VM.weights(cfg, seed=5)
    w["embed"][1] = w["embed"][1] * 8
    T, at = 40, 20
    toks = np.random.default_rng(taps).integers(2, 8, size=T).tolist()
    without = O.forward(raw, w, toks)
    toks[at] = 1
    want = O.forward(raw, w, toks)
    gap = (without - want).pow(2).mean(-1).sqrt() / want.std()
    assert (gap[at:at + taps] > 0.05).all() and (gap[at + taps:] == 0).all() and (gap[:at] == 0).all()
    eng = engine_of(cfg, w, dtype, 6, max_batch=2, max_model_len=128)
    for cuts in ([T], [at + 1, T - at - 1], [at + 1, 2, T - at - 3], [at + 1] + [1] * (T - at - 1), [at + 2, 2, 2, T - at - 6], [1] * T,
                 [2] * 20):
        err = row_errors(feed_all(eng, toks, cuts), want)
        assert float(err.max()) < (1e-5 if dtype == "float32" else 0.02), (cuts, int(err.argmax()), float(err.max()))


def test_a_freed_state_slot_starts_from_zeros():
    """A request in a slot that another one left, whose first portion has one token, two,
    or many: as in a fresh engine."""
    for dtype in ("float32", "bfloat16"):
        eng = engine("edges", dtype, max_batch=1)
        for n in (1, 2, 40):
            feed_all(eng, tokens("edges", 50, seed=n), [20, 30])
            toks = tokens("edges", n + 5, seed=100 + n)
            check(feed_all(eng, toks, [n, 1, 4]), VM.oracle_logits("edges", toks), dtype, f"{n} tokens first")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens(dtype):
    """Sequences of one to four tokens."""
    for name in NAMES:
        eng = engine(name, dtype)
        for n in (1, 2, 3, 4):
            toks = tokens(name, n, seed=40 + n)
            for cuts in ([n], [1] * n):
                check(feed_all(eng, toks, cuts), VM.oracle_logits(name, toks), dtype, f"{name} {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    """300 decoded tokens, over nine page borders and several graph widths."""
    toks = tokens("mixed", 320, seed=9)
    want = VM.oracle_logits("mixed", toks)
    check(feed_all(engine("mixed", dtype), toks, [20] + [1] * 300), want, dtype)


def test_graph_replays_equal_eager_steps():
    """Decode steps of changing batches: every replay gives what the same step gives
    without a graph, with prompts in between."""
    a, b = engine("edges", "bfloat16"), engine("edges", "bfloat16", cuda_graphs=False)
    rng = np.random.default_rng(0)
    ids = [[e.open_feed() for _ in range(4)] for e in (a, b)]
    for step in range(24):
        sel = rng.permutation(4)[:rng.integers(1, 5)]
        toks = {int(i): tokens("edges", 20 if step % 7 == 0 else 1, seed=100 * step + int(i)) for i in sel}
        out = [e.feed([(x[i], t, [len(t) - 1]) for i, t in toks.items()]) for e, x in zip((a, b), ids)]
        assert float(row_errors(out[0], out[1].double().cpu()).max()) < 1e-6, step
    assert a.stats["graph_replays"] > 8 and b.stats["graph_replays"] == 0


def _greedy_ok(name, prompts, outs, dtype):
    for p, r in zip(prompts, outs):
        lg = VM.oracle_logits(name, list(p) + r.output)
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

    if "prefix_caching" in kw and VM.config(name).has_state:
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

    cfg, w = VM.model("mixed")
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

    cfg, w = VM.model("mixed")
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
    wx, wy = (VM.oracle_logits("mixed", toks[k]) for k in "xy")
    read = lambda n: torch.from_numpy(np.fromfile(tmp_path / f"{n}.f32", "<f4")).reshape(-1, cfg.vocab)  # noqa: E731
    check(read(0), wx[[0, 29]], "float32")
    check(read(2), torch.stack([wy[8], wx[39]]), "float32")
    assert not (tmp_path / "1.f32").exists()


def test_serving_benchmark_on_a_model_folder(tmp_path, capsys):
    """The command line, from a checkpoint to generated tokens."""
    from kgs.serve.bench import main
    from kgs.utils.safetensors import save_file

    cfg, w = VM.model("edges")
    (tmp_path / "config.json").write_text(json.dumps(cfg.raw))
    save_file(w, tmp_path / "model.safetensors")
    assert main(["--model", str(tmp_path), "--requests", "5", "--input-len", "33", "--output-len", "6", "--max-batch", "4",
                 "--max-model-len", "256", "--chunked-prefill", "48"]) == 0
    out = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert out["output_tok_per_s"] > 0 and out["stats"]["decode_tokens"] >= 5 * 5
