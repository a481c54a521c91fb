"""Trace runner: feeds given token ids through a model's engine, step by step, and writes the logits asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Standard input brings one JSON object a line: ``{"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}``.  A step
runs the entries' tokens from where their requests stand; ``want`` lists the places among these tokens whose logits
go to DIR/<step>.f32 (little-endian float32 [wanted, vocab], in the order of the entries); the requests in ``end`` give
their slots back.  ``done <step>`` is printed after every step.  Nothing is sampled.

It only drives ``registry.load_engine`` and the engine's ``alloc`` / ``extend`` / ``release``.  Exit code 3: the model's
architecture does not run in the number format.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

SLOTS = 8  # sequences alive at a time


def main(argv=None, stdin=None, stdout=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="Feed given tokens through a model step by step and write logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], required=True)
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    ap.add_argument("--device", default="cuda")
    a = ap.parse_args(argv)
    stdin, stdout = stdin or sys.stdin, stdout or sys.stdout

    from . import _lib, checkpoint, registry

    import torch

    dtype = getattr(torch, a.dtype)
    arch = registry.of_config(checkpoint.read_config(a.model))
    if dtype not in arch.dtypes:
        print(f"trace_run: {arch.name} does not run in {a.dtype}", file=sys.stderr)
        return 3
    _lib.build_missing()
    if dtype == torch.float32:
        torch.set_float32_matmul_precision("highest")
    engine = registry.load_engine(a.model, SLOTS, max(a.max_tokens, 1), device=a.device, dtype=dtype)
    slots = {}
    for line in stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries, want = [], []
        for e in step["entries"]:
            if e["id"] not in slots:
                slots[e["id"]] = engine.alloc()
            if e["tokens"]:
                entries.append((slots[e["id"]], e["tokens"]))
                want.append(e["want"])
        if entries:
            logits = engine.extend(entries, want)
            if logits.shape[0]:
                path = os.path.join(a.out, f"{step['step']}.f32")
                with open(path + ".part", "wb") as f:
                    f.write(logits.float().cpu().contiguous().numpy().astype("<f4").tobytes())
                os.replace(path + ".part", path)
        for i in step.get("end", []):
            if i in slots:
                engine.release(slots.pop(i))
        print(f"done {step['step']}", file=stdout, flush=True)
    return 0
