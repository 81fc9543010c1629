"""Greedy generation from token ids, for every model the registry knows.

    python -m candle_amd.generate --model DIR_OR_GGUF --tokens 1,15,7 --new 32 [--dtype bfloat16|float32] [--ctx 4096]

Prints the generated token ids and the prompt / decode throughput.
"""
from __future__ import annotations

import argparse

from .registry import load_model


def main(argv=None) -> None:
    ap = argparse.ArgumentParser(prog="python -m candle_amd.generate", description="greedy generation from token ids")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors, or a GGUF file")
    ap.add_argument("--tokens", required=True, help="prompt token ids, comma separated")
    ap.add_argument("--new", type=int, default=32, help="tokens to generate")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16", help="precision of the matrix products (folders)")
    ap.add_argument("--ctx", type=int, default=4096, help="positions the caches hold")
    a = ap.parse_args(argv)
    prompt = [int(t) for t in a.tokens.split(",")]
    model = load_model(a.model, dtype=a.dtype, ctx=a.ctx)
    r = model.generate_greedy(prompt, a.new)
    print(",".join(str(t) for t in r["tokens"]))
    print(f"prompt {len(prompt) / r['prompt_seconds']:.1f} tok/s, decode {r['decode_steps'] / max(r['decode_seconds'], 1e-9):.1f} tok/s")


if __name__ == "__main__":
    main()
