"""Generates from a model directory of any kind the engine knows: a layered model (config.json, model.safetensors) or a llama weight
directory (metadata.json).

    python -m espresso_amd.run_model DIR --tokens 1,2,3 [--max-tokens N] [--temperature T --seed S] [--context N] [--precision bf16|f32]
    python -m espresso_amd.run_model DIR --tokenizer TOKENIZER_DIR --prompt TEXT ...

Generated token ids (or text) on standard output, figures of the run on standard error.
"""
from __future__ import annotations

import argparse
import sys


def main(argv: list[str]) -> int:
    ap = argparse.ArgumentParser(prog="run_model", description="Generate from a model directory.")
    ap.add_argument("model", help="model directory")
    ap.add_argument("--tokens", help="prompt token ids, comma separated")
    ap.add_argument("--tokenizer", help="tokenizer directory, for --prompt")
    ap.add_argument("--prompt", help="prompt text")
    ap.add_argument("--max-tokens", type=int, default=32)
    ap.add_argument("--temperature", type=float, default=0.0)
    ap.add_argument("--seed", type=int, default=None, help="sampling seed (temperature > 0)")
    ap.add_argument("--context", type=int, default=4096, help="context length of a layered model")
    ap.add_argument("--eos", type=int, default=None, help="token that ends the generation")
    ap.add_argument("--precision", choices=("bf16", "f32"), default="bf16", help="arithmetic of a layered model")
    a = ap.parse_args(argv)
    if (a.tokens is None) == (a.prompt is None) or (a.prompt is not None and a.tokenizer is None):
        ap.error("give --tokens, or --prompt with --tokenizer")
    from . import engine, ops
    try:
        ops.init()
        cfg = engine.load_model_config(a.model, a.context)
        if a.eos is not None:
            cfg.eos_token = a.eos
        e = engine.RealModelInferenceEngine(cfg, a.model, a.tokenizer, {"ESPRESSO_HIP_PRECISION": a.precision})
        env = {} if a.seed is None else {"ESPRESSO_HIP_SAMPLING_SEED": str(a.seed)}
        if a.prompt is not None:
            text, tokens, r = e.generate_text(a.prompt, a.max_tokens, a.temperature, env)
            print(text)
        else:
            tokens, r = e.generate([int(t) for t in a.tokens.split(",")], a.max_tokens, a.temperature, env)
            print(",".join(map(str, tokens)))
        e.close()
    except Exception as err:
        sys.stderr.write(f"Error: {err}\n")
        return 1
    sys.stderr.write(f"{cfg.name}, {cfg.n_layer} layers, d={cfg.d_model}, vocab={cfg.vocab}: {len(tokens)} tokens, {r['tokens_per_second']:.1f} tok/s, "
                     f"built in {r['compile_time_ms']:.0f} ms\n")
    return 0


if __name__ == "__main__":
    sys.exit(main(sys.argv[1:]))
