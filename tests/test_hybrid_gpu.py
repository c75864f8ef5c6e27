"""Ruruzen through the serving engine on the GPU: small models of other sizes than
each other, against the plain oracle -- whole prompts, token by token, portions,
mixed batches, pages and slots used again, long decoding, generation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

torch = pytest.importorskip("torch")
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

import hybrid_models as HM  # noqa: E402
from oracles import ruruzen as O  # noqa: E402

pytestmark = pytest.mark.gpu

# (median row, worst row): rms over the vocabulary, against the logits' own. In bf16 a
# row whose scores nearly tie moves several times as far as the others.
TOL = {"float32": (3e-6, 2e-5), "bfloat16": (1.6e-2, 8e-2)}
NAMES = sorted(HM.MODELS)


def tokens(name, n, seed=0):
    return np.random.default_rng(seed).integers(0, HM.config(name).vocab, size=n).tolist()


def engine(name, dtype="float32", pages=40, **kw):
    from kgs.serve import EngineConfig, LLMEngine

    cfg = HM.config(name)
    w = HM.weights(cfg)
    object.__setattr__(cfg, "load_weights", lambda seed=0, device="cpu": w)
    kw = {"max_batch": 4, "max_model_len": 1024, **kw}
    return LLMEngine(cfg, EngineConfig(num_pages=pages, dtype=dtype, **kw))


def check(got, want, dtype, what=""):
    got, want = got.detach().cpu().double(), want.double()
    assert got.shape == want.shape
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / want.std()
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
    want = HM.oracle_logits(name, toks)
    eng = engine(name, dtype)
    for cuts in ([T], [1] * T, [2] * 20 + [70], [31, 1, 32, 1, 2, 43], [3, 61, 2, 44], [63, 2, 45], [97, 13]):
        check(feed_all(eng, toks, cuts), want, dtype, f"{name} {cuts[:6]}")
    assert eng.stats["graph_replays"] > 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", NAMES)
def test_residual_after_every_layer(name, dtype):
    cfg = HM.config(name)
    toks = tokens(name, 37, seed=2)
    ref, got = [], []
    O.forward(cfg.raw, {k: v.double() for k, v in HM.weights(cfg).items()}, toks, ref)
    eng = engine(name, dtype)
    eng.model.on_layer = lambda i, x: got.append((i, x.clone()))
    feed_all(eng, toks, [37])
    assert [i for i, _ in got] == list(range(len(cfg.layers)))
    for (i, x), r in zip(got, ref):
        err = (x.cpu().double() - r).pow(2).mean().sqrt() / r.pow(2).mean().sqrt()
        assert err < (2e-6 if dtype == "float32" else 2e-2), (i, float(err))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["odd", "wide"])
def test_unequal_requests_in_one_batch(name, dtype):
    """Portions beside single tokens, a request that waits, one that ends and one
    that takes over its pages and slot: each as if alone."""
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
        check(torch.cat(out[k]), HM.oracle_logits(name, toks[k]), dtype, k)


def test_a_batch_changes_nothing():
    """The same request alone and beside others, on other pages and slots."""
    name = "odd"
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
        a, b = alone.double().cpu(), torch.cat(got).double().cpu()
        assert float((a - b).pow(2).mean().sqrt() / a.std()) < (1e-6 if dtype == "float32" else 1e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("far", [0, 1, 31, 32, 33, 64, 95, 96, 127])
def test_far_key_in_prompt_and_decode(dtype, far):
    """A latent layer whose last query finds one far key by a score that stands out:
    the tokens' embeddings decide, so a key lost or shifted changes the logits."""
    cfg = HM.config("ones")
    raw = json.loads(json.dumps(cfg.raw))
    raw["vocab"], raw["layers"] = 8, [HM.latent(1, 64, 64, 64, 64, 0.3), HM.latent(1, 64, 64, 64, 64, 0.2, kv_from=0)]
    from kgs.models.ruruzen import RuruzenConfig

    cfg = RuruzenConfig.from_dict(raw)
    w = HM.weights(cfg, 3)
    eye = torch.eye(64, dtype=torch.bfloat16)
    g = torch.Generator().manual_seed(1)
    turn = torch.linalg.qr(torch.randn(64, 64, generator=g))[0]
    for n in ("dq", "uq", "dkv", "uv", "o"):
        w["l0.mix." + n] = eye.clone()
    w["l0.mix.uk"] = turn.to(torch.bfloat16)
    w["l0.mix.g"] = w["l0.mix.g"] * 0
    e = torch.randn(8, 64, generator=g)
    e[1] = turn.T @ e[0]        # token 1's key is what token 0 asks for
    w["embed"] = e.to(torch.bfloat16)
    object.__setattr__(cfg, "load_weights", lambda seed=0, device="cpu": w)
    from kgs.serve import EngineConfig, LLMEngine

    T = 131
    toks = np.random.default_rng(far).integers(2, 8, size=T).tolist()
    toks[far], toks[T - 1] = 1, 0
    wd = {k: v.double() for k, v in w.items()}
    want = O.forward(raw, wd, toks)
    without = list(toks)
    without[far] = 2
    gap = (O.forward(raw, wd, without)[-1] - want[-1]).pow(2).mean().sqrt() / want.std()
    assert gap > 0.2  # the far key decides the last logits
    eng = LLMEngine(cfg, EngineConfig(num_pages=12, max_batch=2, max_model_len=256, dtype=dtype))
    for cuts in ([T], [T - 1, 1], [T - 2, 2], [far + 1, T - far - 1] if far + 1 < T else [T], [64, 66, 1]):
        check(feed_all(eng, toks, cuts), want, dtype, f"far {far} {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(dtype):
    """300 decoded tokens, over nine page borders and several graph widths."""
    toks = tokens("odd", 320, seed=9)
    want = HM.oracle_logits("odd", toks)
    check(feed_all(engine("odd", dtype), toks, [20] + [1] * 300), want, dtype)


def _greedy_ok(name, prompts, outs, dtype):
    for p, r in zip(prompts, outs):
        lg = HM.oracle_logits(name, list(p) + r.output)
        for i, t in enumerate(r.output):
            row = lg[len(p) - 1 + i]
            slack = 1e-4 if dtype == "float32" else 0.25
            assert row[t] >= row.max() - slack * row.std(), (len(p), i, t)


@pytest.mark.parametrize("kw", [dict(), dict(chunked_prefill=24), dict(overlap=False), dict(cuda_graphs=False),
                                dict(pages=9, max_model_len=200)], ids=["plain", "chunked", "no-overlap", "eager", "preempt"])
@pytest.mark.parametrize("name", ["odd", "recurrent"])
def test_greedy_generation(name, kw):
    """The engine's own entry point, scheduler and sampler."""
    from kgs.serve import SamplingParams

    eng = engine(name, "float32", **{"max_batch": 3, **kw})
    prompts = [tokens(name, n, seed=n) for n in (1, 33, 60, 7, 64)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=45, ignore_eos=True))
    assert [len(r.output) for r in outs] == [45] * 5
    _greedy_ok(name, prompts, outs, "float32")
    if "pages" in kw:
        assert eng.stats["preemptions"] > 0
    assert eng.sched.check_invariants() == "" and eng.sched.num_running == 0


def test_greedy_generation_bf16_and_sampling():
    from kgs.serve import SamplingParams

    eng = engine("wide", "bfloat16", chunked_prefill=40)
    prompts = [tokens("wide", n, seed=n) for n in (5, 130, 70)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True))
    _greedy_ok("wide", prompts, outs, "bfloat16")
    p = SamplingParams(max_tokens=6, temperature=0.9, top_k=20, top_p=0.9, seed=4, logprobs=2, ignore_eos=True)
    a, b = (eng.generate(prompts, p) for _ in range(2))
    assert [r.output for r in a] == [r.output for r in b] and all(len(r.logprobs) == 6 for r in a)


def test_engine_refuses_what_the_model_has_not():
    from kgs.models.llama import LlamaConfig
    from kgs.serve import EngineConfig, LLMEngine

    for kw in (dict(prefix_caching=True), dict(kv_cache_dtype="fp8"), dict(decode_weights="fp8")):
        with pytest.raises(ValueError):
            engine("odd", **kw)
    with pytest.raises(ValueError, match="bfloat16"):
        LLMEngine(LlamaConfig(hidden=256, heads=2, kv_heads=1, intermediate=256, layers=1, vocab=128),
                  EngineConfig(num_pages=8, max_model_len=64, dtype="float32"))
    eng = engine("odd", pages=4)
    rid = eng.open_feed()
    with pytest.raises(RuntimeError, match="does not fit"):
        eng.feed([(rid, tokens("odd", 200), [])])
    with pytest.raises(ValueError):
        eng.feed([(rid, [1, 2], [2])])
    with pytest.raises(RuntimeError, match="tokens outside"):
        eng.feed([(rid, [203], [])])


def test_trace_run_program(tmp_path):
    """bin/trace_run as a program: steps on standard input, logits in files."""
    _folder(tmp_path)
    toks = {k: tokens("odd", n, seed=n) for k, n in (("x", 40), ("y", 9))}
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks["x"][:30], "want": [0, 29]},
                                     {"id": "y", "tokens": toks["y"][:8], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": toks["y"][8:], "want": []}], "end": ["y"]},
             {"step": 2, "entries": [{"id": "x", "tokens": toks["x"][30:], "want": [9]}], "end": ["x"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "128"], input="\n".join(map(json.dumps, steps)) + "\n",
                       capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-1500:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    assert not (tmp_path / "1.f32").exists()
    got = np.concatenate([np.fromfile(tmp_path / f"{i}.f32", dtype="<f4") for i in (0, 2)]).reshape(3, -1)
    check(torch.from_numpy(got), HM.oracle_logits("odd", toks["x"])[[0, 29, 39]], "float32")


def _folder(tmp_path, name="odd"):
    from kgs.utils.safetensors import save_file

    cfg = HM.config(name)
    (tmp_path / "config.json").write_text(json.dumps(cfg.raw))
    save_file(HM.weights(cfg), tmp_path / "model.safetensors")
    return str(tmp_path)


def test_serving_benchmark_on_a_model_folder(tmp_path, capsys):
    from kgs.serve.bench import main

    assert main(["--model", _folder(tmp_path), "--requests", "5", "--input-len", "33", "--output-len", "6", "--max-batch",
                 "4", "--max-model-len", "256", "--chunked-prefill", "48"]) == 0
    out = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert out["output_tok_per_s"] > 0 and out["stats"]["decode_tokens"] >= 5 * 5


def test_engine_process_serves_a_model_folder(tmp_path):
    """The HTTP server's engine process, started from a model folder's description."""
    import asyncio

    from kgs.models.registry import load_config, to_spec
    from kgs.serve import EngineConfig, SamplingParams
    from kgs.serve.dp import DPEngineLoop

    ec = EngineConfig(num_pages=40, max_batch=2, max_model_len=256, dtype="float32", chunked_prefill=64)
    runner = DPEngineLoop(1, to_spec(load_config(_folder(tmp_path))), ec, device="cuda", start_timeout=100)
    prompt = tokens("odd", 20, seed=3)

    async def one():
        q: asyncio.Queue = asyncio.Queue()
        runner.submit(prompt, SamplingParams(max_tokens=8, ignore_eos=True), asyncio.get_running_loop(), q)
        assert (await q.get())[0] == "id"
        out = []
        while True:
            _, t, fin, _, _ = await q.get()
            out.append(t)
            if fin:
                return out

    try:
        got = asyncio.run(one())
    finally:
        runner.shutdown()

    class R:
        output = got

    _greedy_ok("odd", [prompt], [R], "float32")
