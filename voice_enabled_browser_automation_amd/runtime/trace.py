"""Replay a trace of token ids through a model, step by step, writing logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N < steps

One JSON object a line: {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [0, 1]}], "end": []}.
All entries of a step are one engine step (LLMEngine.step_batch, the call generation makes);
DIR/<step>.f32 receives the wanted rows' f32 logits in order, "done <step>" follows on standard output,
and the requests in "end" give their blocks and state slots back.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, Optional

MAX_LIVE = 4  # requests live at any time (sequence / state slots)


class TraceReplay:
    def __init__(self, model_dir: str, dtype: str, out_dir: str, max_tokens: int, device: str = "cuda"):
        import torch

        from .engine import LLMEngine
        from .weights import load_llm

        # 32-bit: true f32 products everywhere (the kernels', and torch's if one is ever used)
        torch.backends.cuda.matmul.allow_tf32 = False
        model = load_llm(model_dir, device=device, dtype=getattr(torch, dtype))
        block = 16
        blocks = -(-max_tokens // block)
        # (block 0 is the engine's scratch block)
        self.engine = LLMEngine(model, max_seqs=MAX_LIVE, max_model_len=blocks * block, block_size=block,
                                kv_blocks=blocks + 1)
        self.out_dir = out_dir
        self.seqs: Dict[str, object] = {}
        os.makedirs(out_dir, exist_ok=True)

    def step(self, rec: dict) -> None:
        entries, want, n = [], [], 0
        for e in rec["entries"]:
            seq = self.seqs.get(e["id"])
            if seq is None:
                seq = self.seqs[e["id"]] = self.engine.new_sequence([], use_prefix_cache=False)
            entries.append((seq, [int(t) for t in e["tokens"]]))
            want += [n + int(w) for w in e["want"]]
            n += len(e["tokens"])
        logits = self.engine.step_batch(entries, want) if n else None
        if want:
            data = logits.float().cpu().contiguous().numpy().astype("<f4", copy=False)
            path = os.path.join(self.out_dir, f"{rec['step']}.f32")
            with open(path + ".part", "wb") as fh:
                fh.write(data.tobytes())
            os.replace(path + ".part", path)
        for rid in rec.get("end", ()):
            seq = self.seqs.pop(rid, None)
            if seq is not None:
                self.engine.free_sequence(seq, publish=False)


def main(argv: Optional[list] = None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", type=int, required=True, help="most tokens live requests hold at any time")
    ap.add_argument("--device", default="cuda", help="cuda, or cpu for the reference ops")
    a = ap.parse_args(argv)
    if a.device == "cuda":
        from ..ops.build import ensure_kernels

        ensure_kernels()
        import torch

        from .. import ops

        if not torch.cuda.is_available():
            print("trace_run: no GPU", file=sys.stderr)
            return 2
        ops.ext()
    try:
        replay = TraceReplay(a.model, a.dtype, a.out, a.max_tokens, a.device)
    except NotImplementedError as e:  # the model has no kernels for this dtype
        print(f"trace_run: {e}", file=sys.stderr)
        return 3
    for line in sys.stdin:
        if not line.strip():
            continue
        rec = json.loads(line)
        replay.step(rec)
        print(f"done {rec['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
