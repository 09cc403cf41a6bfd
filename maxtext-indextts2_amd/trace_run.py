"""Replays a trace: given token ids go through a model step by step, logits come out (bin/trace_run).

  bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps

Steps are JSON objects, one a line: {"step": n, "entries": [{"id": .., "tokens": [..], "want": [..]}], "end": [ids]}.  The entries of a step are one
batch; for a step in which logits are wanted OUT/<step>.f32 receives them as little-endian f32 [wanted, vocab], and after every step a line
`done <step>` is printed.  Everything runs through MaxEngine.step (StepScheduler): its caches, states and kernels."""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import List

SLOTS = 4            # requests that may be live at a time
PAGE = 64
MAX_ROWS = 4096      # rows of one pass; longer steps run as several


def main(argv: List[str] | None = None) -> int:
  ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids through a model and write logits")
  ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
  ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
  ap.add_argument("--out", required=True, help="folder for the <step>.f32 files")
  ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at a time (pages of 64)")
  args = ap.parse_args(argv)

  from . import build, pyconfig  # pylint: disable=import-outside-toplevel
  build.build()                   # compiles on the first call in a checkout, otherwise returns at once
  from .inference.step_scheduler import StepScheduler  # pylint: disable=import-outside-toplevel
  from .maxengine import MaxEngine  # pylint: disable=import-outside-toplevel

  pages = -(-args.max_tokens // PAGE)
  config = pyconfig.initialize(
      ["trace_run", os.path.join(pyconfig.PKG_DIR, "configs", "base.yml")], ixt_model_dir=args.model, dtype=args.dtype, attention="paged", scan_layers=False,
      per_device_batch_size=float(SLOTS), max_target_length=pages * PAGE, max_prefill_predict_length=min(pages * PAGE, MAX_ROWS), pagedattn_tokens_per_page=PAGE,
      pagedattn_num_pages=pages + 1, use_chunked_prefill=True)     # + 1: page 0 is reserved by the page manager
  engine = MaxEngine(config)
  engine.load_params()
  scheduler = StepScheduler(engine)
  os.makedirs(args.out, exist_ok=True)
  for line in sys.stdin:
    if not line.strip():
      continue
    step = json.loads(line)
    entries = [(e["id"], e["tokens"], e.get("want", [])) for e in step["entries"]]
    if entries:
      logits, _ = scheduler.step(entries)
      if logits is not None and logits.shape[0] > 0:
        logits.cpu().numpy().astype("<f4").tofile(os.path.join(args.out, f"{step['step']}.f32"))
    for request in step.get("end", []):
      scheduler.release(request)
    print(f"done {step['step']}", flush=True)
  engine.close()
  return 0


if __name__ == "__main__":
  sys.exit(main())
