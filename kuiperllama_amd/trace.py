"""Replays a trace of token ids through a model, step by step, and writes the logits that are asked for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N  < steps.jsonl

One JSON object per input line: {"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}.  The entries of a
step are one batch (KuiperModel.forward); a request keeps its sequence slot from its first step until it is named in
"end".  Wanted logits go to DIR/<step>.f32 (little-endian fp32, [wanted, vocab]); every step is acknowledged on
standard output with "done <step>".
"""
from __future__ import annotations

import argparse
import json
import os
import sys


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.splitlines()[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens that live requests hold at any time")
    a = ap.parse_args(argv)
    from . import build
    build.build_lib()
    from .model import KuiperModel
    m = KuiperModel.from_checkpoint(a.model, max_seq_len=a.max_tokens, dtype=a.dtype, max_seqs=min(a.max_tokens, 256))
    live = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        st = json.loads(line)
        entries = []
        for e in st["entries"]:
            if e["id"] not in live:
                live[e["id"]] = m.open_seq()
            entries.append((live[e["id"]], e["tokens"], e["want"]))
        if entries:
            z = m.forward(entries)
            if z.shape[0]:
                z.astype("<f4", copy=False).tofile(os.path.join(a.out, f"{st['step']}.f32"))
        for i in st.get("end", []):
            m.close_seq(live.pop(i))
        print(f"done {st['step']}", flush=True)
    m.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
