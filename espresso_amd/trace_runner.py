"""Replays a trace of token ids through a model directory, step by step, and writes the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps arrive on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

A request's tokens continue its sequence; `want` lists places among the step's tokens whose logits go to OUT/<step>.f32
(little-endian fp32, [wanted, vocab], in the order of the entries); requests listed in `end` give their sequence slot back after the
step.  "done <step>" on standard output answers each step.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

import numpy as np

MAX_LIVE_REQUESTS = 8


def run(model, lines, out_dir: str, vocab: int, answer) -> None:
    """Feeds the steps to `model` (append / acquire_sequence / release_sequence)."""
    live: dict[str, int] = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for entry in step["entries"]:
            want = entry.get("want", [])
            if entry["id"] not in live:
                live[entry["id"]] = model.acquire_sequence()
            if not entry["tokens"]:
                continue
            order = sorted(set(want))
            logits = model.append(entry["tokens"], order, sequence=live[entry["id"]])
            rows += [logits[order.index(w)] for w in want]
        if rows:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            np.stack(rows).astype("<f4").tofile(path + ".part")
            os.replace(path + ".part", path)
        for name in step.get("end", []):
            if name in live:
                model.release_sequence(live.pop(name))
        answer(f"done {step['step']}")


def engine_kind(model_dir: str) -> str:
    """"layered" for a directory with a config.json, "llama" for one with metadata.json."""
    return "layered" if os.path.exists(os.path.join(model_dir, "config.json")) else "llama"


def main(argv: list[str]) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Feed given token ids through a model and write logits.")
    ap.add_argument("--model", required=True, help="model directory (config.json, model.safetensors)")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), required=True)
    ap.add_argument("--out", required=True, help="directory for <step>.f32 files")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    a = ap.parse_args(argv)
    from . import _lib, engine, ops
    if engine_kind(a.model) == "llama" and a.dtype == "float32":
        sys.stderr.write("trace_run: llama runtimes have no all-32-bit arithmetic\n")
        return 3
    if engine_kind(a.model) == "layered":
        _lib.load_library("layered")   # in a checkout with nothing built, this part of the library is all the model needs
    ops.init()
    cfg = engine.load_model_config(a.model, a.max_tokens)
    env = {"ESPRESSO_HIP_PRECISION": "f32" if a.dtype == "float32" else "bf16", "ESPRESSO_HIP_MAX_SEQUENCES": str(MAX_LIVE_REQUESTS)}
    model = engine.RealModelInferenceEngine(cfg, a.model, environment=env).runtime()

    def answer(text: str) -> None:
        sys.stdout.write(text + "\n")
        sys.stdout.flush()

    run(model, sys.stdin, a.out, cfg.vocab, answer)
    return 0
