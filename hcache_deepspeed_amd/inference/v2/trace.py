"""Trace replay: given token ids go through a served model, one ragged batch a step, and chosen logits go to files.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps.jsonl

Standard input holds a step per line, a JSON object that becomes one call of the engine's ``put``:

    {"step": 7, "entries": [{"id": "r1", "tokens": [11, 4], "want": [1]}, {"id": "r2", "tokens": [9]}], "end": ["r1"]}

``want`` are places among an entry's tokens; the logits there, as little-endian float32 rows in entry and ``want`` order,
are written to ``OUT/<step>.f32``. Requests in ``end`` are flushed after the step. ``done <step>`` on standard output
answers each step. ``--max-tokens`` and ``--max-requests`` size the KV pool and the state slots; nothing is sampled."""
import argparse
import json
import os
import sys


def build_engine(model_dir, dtype, max_tokens, max_requests=4, block_size=64, device=None):
    from .engine import build_hf_engine
    blocks = -(-max_tokens // block_size)
    conf = {"dtype": {"bfloat16": "bf16", "float32": "fp32"}[dtype],
            "state_manager": {"max_context": blocks * block_size, "max_ragged_batch_size": blocks * block_size,
                              "max_tracked_sequences": max_requests, "kv_block_size": block_size}}
    return build_hf_engine(model_dir, conf, device=device, num_kv_blocks=blocks)


def run_step(engine, step, out_dir):
    """One step; returns the logits [wanted, vocab] (float32, host) or None."""
    import torch
    logits = None
    entries = step.get("entries") or []
    if entries:
        wanted = [list(e.get("want") or []) for e in entries]
        got, _ = engine.put([e["id"] for e in entries], [torch.tensor(e["tokens"], dtype=torch.int64) for e in entries],
                            capture_latents=False, logits_at=wanted)
        if any(wanted):
            logits = got.float().cpu()
            path = os.path.join(out_dir, f"{step['step']}.f32")
            with open(path, "wb") as f:
                f.write(logits.numpy().astype("<f4").tobytes())
    for uid in step.get("end") or []:
        engine.flush(uid)
    return logits


def _load_needed_kernels(model_dir):
    """Compile (first call of a checkout) only the kernels the model's class runs on."""
    from ...ops import native
    from .arch import spec_from_hf
    from .engine import transformer_class
    with open(os.path.join(model_dir, "config.json")) as f:
        spec = spec_from_hf(json.load(f))
    native.load_kernels(only=getattr(transformer_class(spec), "KERNEL_SOURCES", None))


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a token trace through the serving engine.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, required=True, help="size of the KV pool in tokens (rounded up to pages)")
    ap.add_argument("--max-requests", type=int, default=4, help="state slots")
    args = ap.parse_args(argv)
    import torch
    if not torch.cuda.is_available():
        print("trace_run: no GPU", file=sys.stderr)
        return 2
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")
    _load_needed_kernels(args.model)
    engine = build_engine(args.model, args.dtype, args.max_tokens, args.max_requests)
    os.makedirs(args.out, exist_ok=True)
    for line in sys.stdin:
        if line.strip():
            step = json.loads(line)
            run_step(engine, step, args.out)
            print(f"done {step['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
