"""Replay given token steps through the engine and write logits.

One JSON object a line on standard input:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3],
                             "want": [0, 2]}], "end": ["b"]}

All entries of a step are one batch: each runs its tokens on top of what
earlier steps left in the cache. The logits at the wanted places go to
OUT/<step>.f32 (little-endian fp32, [wanted, vocab]); "end" lists requests
whose pages are given back after the step. After every step the line
"done <step>" is printed. Sampling is the only part of the generation path
that does not run.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

BLOCK_SIZE = 16
MAX_LIVE = 4


def make_engine(model: str, dtype: str, max_tokens: int,
                device: str = "cuda:0"):
    """An engine whose pool holds max_tokens tokens of MAX_LIVE requests."""
    from helix_amd.engine.engine import EngineConfig, LLMEngine
    tokens = -(-max_tokens // BLOCK_SIZE) * BLOCK_SIZE
    return LLMEngine(EngineConfig(
        model=model, dtype=dtype, block_size=BLOCK_SIZE,
        max_num_seqs=MAX_LIVE, max_model_len=tokens,
        kv_cache_blocks=tokens // BLOCK_SIZE,
        enable_prefix_caching=False), device=device)


def run_step(engine, step: dict, out_dir: str) -> None:
    entries = [(e["id"], e["tokens"], e.get("want", []))
               for e in step.get("entries", [])]
    logits = engine.extend(entries) if entries else None
    if logits is not None:
        data = logits.float().cpu().numpy().astype("<f4", copy=False)
        with open(os.path.join(out_dir, f"{step['step']}.f32"), "wb") as f:
            f.write(data.tobytes())
    for sid in step.get("end", []):
        engine.release(sid)


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(
        prog="trace_run", description="Replay token steps from standard "
        "input through the engine and write their logits.")
    ap.add_argument("--model", required=True,
                    help="folder with config.json and safetensors")
    ap.add_argument("--dtype", default="bfloat16",
                    choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="tokens that live requests hold at most")
    ap.add_argument("--device", default="cuda:0")
    args = ap.parse_args(argv)

    if args.device.startswith("cuda"):
        from helix_amd.models import registry
        from helix_amd.ops import build
        build.ensure(registry.model_class(
            registry.get_config(args.model)).extension)
    os.makedirs(args.out, exist_ok=True)
    engine = make_engine(args.model, args.dtype, args.max_tokens,
                         args.device)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        run_step(engine, step, args.out)
        print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
