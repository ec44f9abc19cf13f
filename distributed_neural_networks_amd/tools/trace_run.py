"""``bin/trace_run``: feed given token ids through a model and write logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

Each step is one batch of the engine (``runtime/engine.py``).  For a step that
wants logits, ``DIR/<step>.f32`` receives them ([wanted, vocab], little-endian
fp32, in the order of the entries and of ``want``); ``done <step>`` is printed
after every step.  The cache pool holds ``--max-tokens`` tokens, every live
sequence rounded up to whole pages, and up to four sequences are live at a time.

The kernels are compiled at the first call in a fresh checkout.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import List, Optional

MAX_LIVE = 4


def parse_args(argv: Optional[List[str]] = None):
    p = argparse.ArgumentParser(prog="trace_run", description="Replay a token trace through a model; writes logits.")
    p.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    p.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    p.add_argument("--out", required=True, help="folder for <step>.f32")
    p.add_argument("--max-tokens", type=int, required=True, help="tokens the cache pool holds")
    a = p.parse_args(argv)
    if a.max_tokens < 1:
        p.error("--max-tokens must be positive")
    return a


def build_engine(folder: str, dtype: str, max_tokens: int):
    """Engine over one stage with the whole model of ``folder``."""
    import torch
    from .. import checkpoint as ckpt
    from ..models import model_info
    from ..runtime.engine import Engine
    from ..runtime.paging import pages_for
    from ..runtime.transformer import build_device_stage
    info = model_info(folder)
    n = info.num_layers
    sd = ckpt.stage_state_dict(info.name, ckpt.load_full_state_dict(folder), 0, n - 1, True, True)
    stage = build_device_stage(info.name, sd, 0, n - 1, True, True, torch.device("cuda", 0), dtype=dtype,
                               max_batch=1, max_seq=max_tokens, max_tokens=max_tokens,
                               num_pages=pages_for(max_tokens), num_slots=MAX_LIVE)
    return Engine([stage], max_slots=MAX_LIVE)


def run(engine, lines, out: str) -> None:
    from ..runtime.engine import Entry
    for line in lines:
        if not line.strip():
            continue
        s = json.loads(line)
        logits = engine.step([Entry(e["id"], e["tokens"], e.get("want") or ()) for e in s["entries"]])
        if logits is not None:
            data = logits.float().cpu().contiguous().numpy().astype("<f4", copy=False).tobytes()
            with open(os.path.join(out, f"{s['step']}.f32"), "wb") as f:
                f.write(data)
        for i in s.get("end") or ():
            engine.end(i)
        print(f"done {s['step']}", flush=True)


def main(argv: Optional[List[str]] = None) -> int:
    a = parse_args(argv)
    from ..ops import build
    build.ensure("decoder")
    engine = build_engine(a.model, a.dtype, a.max_tokens)
    os.makedirs(a.out, exist_ok=True)
    run(engine, sys.stdin, a.out)
    return 0
