"""Feeds given token ids through a model step by step and writes the logits. Samples nothing.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line:
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
All entries of a step run as one batch through the framework's own model, step function, cache
and kernels. For a step in which something is wanted, OUT/<step>.f32 holds the logits at the
wanted places ([wanted, vocab] little-endian float32, in the order of the entries and of
``want``). After every step a line ``done <step>`` is printed. The reference's counterpart is
scripts/golden_logits.py (teacher-forced logits saved for later comparison).

With --hidden-out DIR every step also leaves the residual stream of all its tokens (in the order
of the entries) after the embedding, DIR/<step>.embedding.f32, and after each layer,
DIR/<step>.<layer>.f32, as [tokens, width] float32: for finding the layer at which a difference
starts (the reference hands out its blocks' outputs for that: engine/include/gpt2_gpu.h:21-25).

``main`` is the whole program; ``steps`` and ``out`` stand in for standard input and output."""

from __future__ import annotations

import argparse
import json
import sys
from pathlib import Path


def main(argv=None, steps=None, out=None) -> int:
    parser = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n")[0])
    parser.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    parser.add_argument("--dtype", required=True, choices=("bfloat16", "float32"))
    parser.add_argument("--out", required=True, help="folder for the <step>.f32 files")
    parser.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time")
    parser.add_argument("--page-size", type=int, default=None, help="tokens per cache page (default: the engine's)")
    parser.add_argument("--max-requests", type=int, default=4, help="requests that are live at any time: the cache has as many state slots")
    parser.add_argument("--hidden-out", default=None, help="folder for the residual stream after the embedding and after each layer")
    args = parser.parse_args(argv)

    from ..engine import ModelRunner, StepEntry
    from ..engine.loading import DEFAULT_PAGE_SIZE, load_model, make_cache
    from ..ops import library

    library()  # builds the kernels now if this is a fresh checkout, and fails loudly if it cannot
    device = "cuda:0"
    model = load_model(args.model, args.dtype, device)
    page_size = args.page_size or DEFAULT_PAGE_SIZE
    # --max-tokens counts every live request rounded up to a multiple of 64. With larger pages each
    # of those 64-token units may be a request of its own that needs a whole page.
    max_tokens = args.max_tokens if page_size <= 64 else -(-args.max_tokens // 64) * page_size
    # a model without a position limit of its own: no request can hold more than the pool does
    max_length = model.max_positions() or -(-max_tokens // page_size) * page_size
    cache = make_cache(model, max_tokens=max_tokens, page_size=page_size, max_requests=args.max_requests, device=device, max_length=max_length)
    runner = ModelRunner(model, cache, device)
    out_dir = Path(args.out)
    out_dir.mkdir(parents=True, exist_ok=True)
    hidden_dir = Path(args.hidden_out) if args.hidden_out else None
    if hidden_dir is not None:
        hidden_dir.mkdir(parents=True, exist_ok=True)

    for line in sys.stdin if steps is None else steps:
        line = line.strip()
        if not line:
            continue
        record = json.loads(line)
        step = record["step"]
        entries = [StepEntry(e["id"], [int(t) for t in e["tokens"]], [int(w) for w in e.get("want", [])]) for e in record.get("entries", [])]
        for entry in entries:
            if not cache.has(entry.request_id):
                cache.open(entry.request_id)
        if entries:
            observer = None
            if hidden_dir is not None:
                observer = lambda name, rows: rows.cpu().numpy().astype("<f4", copy=False).tofile(hidden_dir / f"{step}.{name}.f32")
            logits = runner.step(entries, observer=observer)
            if logits is not None:
                logits.cpu().numpy().astype("<f4", copy=False).tofile(out_dir / f"{step}.f32")
        for request_id in record.get("end", []):
            if cache.has(request_id):
                cache.close(request_id)
        print(f"done {step}", file=out or sys.stdout, flush=True)
    runner.drop_graphs()
    return 0


if __name__ == "__main__":
    sys.exit(main())
