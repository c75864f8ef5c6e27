"""Replay of a token trace through the serving engine: requests' tokens are given
step by step on standard input, the logits asked for are written to files.

  bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Each input line is one step, a JSON object ``{"step": n, "entries": [{"id", "tokens",
"want"}, ...], "end": [ids]}``: all entries run as one batch (:meth:`LLMEngine.feed`),
the logits at the wanted places go to ``DIR/<n>.f32`` (little-endian fp32, [wanted,
vocab]), the requests in ``end`` give back what they hold, and ``done <n>`` is
printed. The cache pool holds N tokens (in whole pages), with state slots for
four requests. Exit code 3: the model has no 32-bit path.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

LIVE_REQUESTS = 4


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time")
    a = ap.parse_args(argv)
    from kgs.models.registry import load_config, of_config
    from kgs.ops.decode import PAGE

    from .engine import EngineConfig, LLMEngine

    cfg = load_config(a.model)
    if a.dtype not in getattr(of_config(cfg).serving_class(), "DTYPES", ("bfloat16",)):
        return 3
    pages = -(-a.max_tokens // PAGE)
    eng = LLMEngine(cfg, EngineConfig(num_pages=pages + 1, max_batch=LIVE_REQUESTS, max_model_len=pages * PAGE,
                                      dtype=a.dtype))
    live: dict = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            if e["id"] not in live:
                live[e["id"]] = eng.open_feed()
            entries.append((live[e["id"]], e["tokens"], e["want"]))
        logits = eng.feed(entries)
        if logits.shape[0]:
            path = os.path.join(a.out, f"{step['step']}.f32")
            logits.float().cpu().numpy().astype("<f4").tofile(path)
        for rid in step["end"]:
            if rid in live:
                eng.close_feed(live.pop(rid))
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    raise SystemExit(main())
