"""Command line: `bin/generate` (sample from a model folder) and `bin/trace_run` (replay token traces, write logits)."""
from __future__ import annotations

import argparse
import json
import os
import subprocess
import sys

from . import _lib


def ensure_library() -> None:
    """Builds the HIP library when the checkout has none (hipcc, no GPU needed)."""
    if not _lib.built():
        build = os.path.join(os.path.dirname(_lib._HERE), "build.py")
        subprocess.run([sys.executable, build, "--serving"], check=True, stdout=sys.stderr)


def _load(args, num_blocks, max_batch):
    from .registry import load_model
    return load_model(args.model, dtype=args.dtype, num_blocks=num_blocks, max_batch=max_batch)


def _common(description):
    ap = argparse.ArgumentParser(description=description)
    ap.add_argument("--model", required=True, metavar="DIR", help="folder with config.json and the checkpoint")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    return ap


def replay(model, steps, out_dir, done) -> None:
    """Runs trace steps -- {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]} -- through model.step.  For a step
    that wants logits, writes out_dir/<n>.f32: rows of little-endian fp32, in the order of the entries and of their `want`
    (places among the entry's tokens).  Calls done(n) after every step; ended requests give their blocks back first."""
    live = {}
    for st in steps:
        sids, tokens, rows, base = [], [], [], 0
        for e in st["entries"]:
            if not e["tokens"]:
                if e.get("want"):
                    raise ValueError(f"request {e['id']} wants logits of a step that brings no tokens for it")
                continue
            if e["id"] not in live:
                live[e["id"]] = model.new_sequence()
            sids.append(live[e["id"]])
            tokens.append(e["tokens"])
            for w in e.get("want", []):
                if not 0 <= w < len(e["tokens"]):
                    raise ValueError(f"request {e['id']}: place {w} is not among its {len(e['tokens'])} tokens")
                rows.append(base + w)
            base += len(e["tokens"])
        if sids:
            logits = model.step(sids, tokens, rows=rows)
            if rows:
                logits.cpu().numpy().astype("<f4").tofile(os.path.join(out_dir, f"{st['step']}.f32"))
        for rid in st.get("end", []):
            if rid in live:
                model.free_sequence(live.pop(rid))
        done(st["step"])


def trace_main(argv=None) -> int:
    ap = _common("Replays token traces, read from standard input one JSON step a line, and writes the logits that they ask for.")
    ap.add_argument("--out", required=True, metavar="DIR", help="where <step>.f32 files go")
    ap.add_argument("--max-tokens", type=int, required=True, metavar="N", help="most tokens that live requests hold at any time")
    args = ap.parse_args(argv)
    ensure_library()
    import torch
    from .engine import BLOCK
    from .registry import UnsupportedDtype
    max_batch = 64
    # every live request may leave its last block partly empty
    blocks = (args.max_tokens + BLOCK - 1) // BLOCK + max_batch
    with torch.no_grad():
        try:
            model = _load(args, blocks, max_batch)
        except UnsupportedDtype as e:
            print(e, file=sys.stderr)
            return 3
        os.makedirs(args.out, exist_ok=True)
        steps = (json.loads(line) for line in sys.stdin if line.strip())
        replay(model, steps, args.out, lambda n: print(f"done {n}", flush=True))
    return 0


def generate_main(argv=None) -> int:
    ap = _common("Generates from prompts of token ids, all prompts as one batch; prints one JSON list of new ids per prompt.")
    ap.add_argument("--prompt", action="append", required=True, metavar="'ID ID ...'", help="token ids (repeat for a batch)")
    ap.add_argument("--max-new-tokens", type=int, default=32)
    ap.add_argument("--temperature", type=float, default=1.0, help="0: greedy")
    ap.add_argument("--top-k", type=int, default=None)
    ap.add_argument("--eos", type=int, default=None, metavar="ID")
    ap.add_argument("--seed", type=int, default=0)
    args = ap.parse_args(argv)
    ensure_library()
    import torch
    from .engine import BLOCK
    prompts = [[int(t) for t in p.replace(",", " ").split()] for p in args.prompt]
    blocks = sum((len(p) + args.max_new_tokens + BLOCK - 1) // BLOCK for p in prompts)
    model = _load(args, blocks, len(prompts))
    gen = torch.Generator(device=model.device).manual_seed(args.seed)
    for ids in model.generate_batch(prompts, args.max_new_tokens, args.temperature, args.top_k, args.eos, generator=gen):
        print(json.dumps(ids))
    return 0
