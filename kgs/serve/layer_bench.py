"""Prefill and decode throughput of a Ruruzen, Nufusun, Nokipel or Vumalix layer stack at sizes
that resemble a real model's layers (random weights), beside stacks of the closest other
models of the same width, heads, feed-forward (where there are experts: those that a token
uses) and depth: ``python bench.py --workload ruruzen|nufusun|nokipel|vumalix``.

All run through :class:`LLMEngine`'s own step runners: prefill a whole prompt
batch in one step, decode a hipGraph replay per step. Per case the median of
several interleaved rounds (one of each model in turn) is reported.
"""
from __future__ import annotations

import statistics
from types import SimpleNamespace

import numpy as np
import torch

from kgs.models.llama import LlamaConfig
from kgs.models.nokipel import NokipelConfig
from kgs.models.nufusun import NufusunConfig
from kgs.models.ruruzen import RuruzenConfig
from kgs.models.vumalix import VumalixConfig
from kgs.ops.decode import PAGE

# name -> width, heads, q_rank, kv_rank, ff, Llama kv heads (head size 128 everywhere)
SIZES = {"w2048": (2048, 16, 768, 512, 8192, 4), "w4096": (4096, 32, 1536, 512, 14336, 8)}
EXPERTS, TOP = 16, 4     # experts of a layer and those a token uses, together as wide as ff
IDENTITY = 2             # Nokipel: identity experts among them; one of the TOP is the shared expert
ATTENTION_CHUNK = 5120   # Nokipel: positions of an attention chunk (3072 keys at the longest context below)
WINDOW, ROT_DIM, TAPS = 2048, 64, 3  # Vumalix: of its latent attention, and of its convolutions
LAYERS = {"ruruzen": "LDSD", "nufusun": "AAAA", "nokipel": "LAMC", "vumalix": "LASA"}
BESIDE = {"ruruzen": ("llama",), "nufusun": ("llama",), "nokipel": ("nufusun", "ruruzen"), "vumalix": ("ruruzen", "nokipel")}
VOCAB = 32000
PREFILL = ((1, 8192), (8, 1024), (64, 128))              # sequences x tokens
DECODE = ((1, 1024), (16, 1024), (64, 1024), (256, 1024), (16, 8192))  # batch x context


def ruruzen(size: str, layers: str) -> RuruzenConfig:
    """``layers``: one letter per layer -- L latent attention, S latent attention
    reading the first L's latent, D delta rule; all with a feed-forward."""
    width, heads, qr, kr, ff, _ = SIZES[size]
    out = []
    for ch in layers:
        if ch == "D":
            e = {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": heads, "dim": 128, "vdim": 128, "conv": 4}}
        else:
            e = {"type": "latent_attention", "mixer": {"heads": heads, "dim": 128, "vdim": 128, "q_rank": qr,
                                                       "kv_rank": kr, "scale": 128 ** -0.5}}
            if ch == "S":
                e["mixer"]["kv_from"] = layers.index("L")
        out.append({**e, "mlp": {"kind": "dense", "ff": ff}})
    return RuruzenConfig.from_dict({"architecture": "Ruruzen", "vocab": VOCAB, "width": width, "streams": 4,
                                    "logit_softcap": 30.0, "norm": {"eps": 1e-5}, "layers": out})


def nufusun(size: str, layers: str) -> NufusunConfig:
    """``layers``: one letter per layer -- A attention and experts, N attention alone."""
    width, heads, _, _, ff, kv = SIZES[size]
    mixer = {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "bias_max": 128}
    mlp = {"kind": "moe", "router": {"experts": EXPERTS, "top": TOP}, "expert": {"ff": ff // TOP, "limit": 7.0}}
    return NufusunConfig.from_dict({
        "architecture": "Nufusun", "vocab": VOCAB, "width": width, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5},
        "layers": [{"type": "attention", "mixer": mixer, "mlp": mlp if ch == "A" else None} for ch in layers]})


def nokipel(size: str, layers: str) -> NokipelConfig:
    """``layers``: one letter per layer -- L lightning attention and a dense feed-forward,
    M lightning attention and experts, C chunked attention and a dense feed-forward, A
    chunked attention and experts."""
    width, heads, _, _, ff, kv = SIZES[size]
    attention = {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                 "mask": {"size": ATTENTION_CHUNK}, "rot": {"dims": 64, "base": 5e5}}
    lightning = {"heads": heads, "dim": 128, "vdim": 128, "decay": [1 - 2.0 ** -(1 + 9 * i / heads) for i in range(heads)]}
    dense = {"kind": "dense", "ff": ff, "limit": 7.0}
    moe = {"kind": "moe", "expert": {"ff": ff // TOP}, "shared": {"ff": ff // TOP},
           "router": {"experts": EXPERTS - IDENTITY, "identity": IDENTITY, "top": TOP - 1, "scale": 1.5,
                      "groups": {"count": 4, "keep": 2}}}
    kinds = {"L": ("lightning", lightning, dense), "M": ("lightning", lightning, moe),
             "C": ("attention", attention, dense), "A": ("attention", attention, moe)}
    return NokipelConfig.from_dict({
        "architecture": "Nokipel", "vocab": VOCAB, "width": width, "embedding": {"scale": 1.0},
        "norm": {"eps": 1e-5, "groups": 8},
        "layers": [dict(zip(("type", "mixer", "mlp"), kinds[ch])) for ch in layers]})


def vumalix(size: str, layers: str) -> VumalixConfig:
    """``layers``: one letter per layer -- L latent attention, S latent attention with the
    first L's weights, A differential attention (maps half as wide as a value, so that its
    cache is as large as other designs'); all with a feed-forward."""
    width, heads, qr, kr, ff, kv = SIZES[size]
    latent = {"heads": heads, "dim": 128, "rot_dim": ROT_DIM, "vdim": 128, "q_rank": qr, "kv_rank": kr,
              "scale": (128 + ROT_DIM) ** -0.5, "mask": {"size": WINDOW}, "rot": {"dims": ROT_DIM, "base": 1e4}}
    attention = {"heads": heads, "kv_heads": kv, "dim": 64, "vdim": 128, "scale": 64 ** -0.5, "diff": 0.7,
                 "q_temp": {"coef": 0.1, "every": 4096}}
    out = []
    for ch in layers:
        e = {"type": "attention", "mixer": attention} if ch == "A" else {"type": "latent_attention", "mixer": latent}
        if ch == "S":
            e["weights_of"] = layers.index("L")
        out.append({**e, "mlp": {"kind": "dense", "ff": ff}})
    return VumalixConfig.from_dict({"architecture": "Vumalix", "vocab": VOCAB, "width": width, "norm": {"eps": 1e-5},
                                    "canon": {"taps": TAPS}, "layers": out})


def llama(size: str, layers: str) -> LlamaConfig:
    width, heads, _, _, ff, kv = SIZES[size]
    return LlamaConfig(hidden=width, intermediate=ff, heads=heads, kv_heads=kv, layers=len(layers), vocab=VOCAB)


def _plan(nseq: int, n: int, pos0: int, decode: bool, state: bool, pad: int, rng) -> SimpleNamespace:
    """A scheduler plan of ``nseq`` sequences with scattered pages."""
    per = -(-(pos0 + n) // PAGE)
    pages = (1 + rng.permutation(nseq * per)).reshape(nseq, per).astype(np.int32)
    padded = n if decode else -(-n // pad) * pad
    pos = pos0 + np.arange(padded)
    real = np.arange(padded) < n
    slots = np.where(real[None], pages[:, np.minimum(pos // PAGE, per - 1)] * PAGE + pos % PAGE, -1).reshape(-1)
    e = np.zeros(0, np.int32)
    p = SimpleNamespace(seq_ids=np.arange(nseq), tokens=rng.integers(0, VOCAB, nseq * padded).astype(np.int32),
                        positions=np.tile(pos, nseq).astype(np.int32), slots=slots.astype(np.int32),
                        state_slots=(1 + rng.permutation(nseq)).astype(np.int32) if state else e)
    if decode:
        p.kind, p.n_prefill, p.block_tables, p.max_pages = 2, 0, pages, per
        p.ctx_lens = np.full(nseq, pos0 + 1, np.int32)
        p.seq_lens = p.seq_starts = p.ctx_starts = p.last_chunk = e
        p.pf_max_pages = 0
    else:
        p.kind, p.n_prefill, p.pf_block_tables, p.pf_max_pages = 1, nseq, pages, per
        p.seq_lens = np.full(nseq, n, np.int32)
        p.padded_lens = np.full(nseq, padded, np.int32)
        p.seq_starts = (np.arange(nseq) * padded).astype(np.int32)
        p.ctx_starts, p.last_chunk = np.zeros(nseq, np.int32), np.ones(nseq, np.uint8)
        p.max_pages, p.ctx_lens = 0, e
    return p


def _time(run, steps: int) -> float:
    """Milliseconds per call of ``steps`` back-to-back calls."""
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(steps):
        run()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / steps


def run(sizes=("w2048", "w4096"), layers: str = "LDSD", rounds: int = 3, prefill=PREFILL, decode=DECODE,
        models=("ruruzen", "llama"), progress=lambda s: None) -> list[dict]:
    """``models``: "ruruzen", "nufusun", "nokipel", "vumalix", "llama"; ``layers``: the first one's, a
    further design has its own."""
    from .engine import EngineConfig, LLMEngine

    out = []
    for size in sizes:
        most = max([b * (c + 1) for b, c in decode] + [b * (c + 128) for b, c in prefill])
        nb = max([b for b, _ in decode] + [b for b, _ in prefill])
        ec = dict(num_pages=most // PAGE + 2 * nb + 2, max_batch=max(256, nb), max_model_len=16384)
        engines = {}
        for m in models:
            make = {"ruruzen": ruruzen, "nufusun": nufusun, "nokipel": nokipel, "vumalix": vumalix, "llama": llama}[m]
            cfg = make(size, layers if m in (models[0], "llama") else LAYERS[m])
            engines[m] = LLMEngine(cfg, EngineConfig(**ec))
            progress(f"{size} {m} ready")
        for kind, cases in (("prefill", prefill), ("decode", decode)):
            for b, n in cases:
                rng = np.random.default_rng(b + n)
                runs = {}
                for m, eng in engines.items():
                    dec = kind == "decode"
                    p = _plan(b, 1 if dec else n, n if dec else 0, dec, eng.model.has_state, eng.model.pad_multiple, rng)
                    eng._check_plan(p)
                    step = eng._run_decode if dec else eng._run_prefill
                    runs[m] = lambda step=step, p=p: step(p)
                    for _ in range(3):
                        runs[m]()
                    torch.cuda.synchronize()
                k = 50 if kind == "decode" else 5
                ms = {m: [] for m in runs}
                for _ in range(rounds):
                    for m, r in runs.items():
                        ms[m].append(_time(r, k))
                row = {"size": size, "layers": layers, "step": kind, "sequences": b,
                       ("context" if kind == "decode" else "tokens"): n}
                for m, t in ms.items():
                    t = statistics.median(t)
                    row[m] = {"ms": round(t, 4), "tok_per_s": round(b * (1 if kind == "decode" else n) / t * 1e3, 1)}
                out.append(row)
                progress(f"{row}")
                for eng in engines.values():
                    eng._graphs.clear()
        del engines
        torch.cuda.empty_cache()
    return out
