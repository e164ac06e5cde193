"""Command-line generation with any language model of the framework.

    python -m voice_enabled_browser_automation_amd.generate --model DIR --ids 5,17,3 --ids 8,9 --max-new 32
    python -m voice_enabled_browser_automation_amd.generate --model llama3.2-1b --tokenizer llama3 --text "open the page"

--model: a checkpoint folder (config.json + safetensors) or a preset (random weights).  Prompts are
token ids, or text with --tokenizer; every prompt is a request of one continuous batch
(runtime/scheduler.py).  One JSON line per prompt on standard output.
"""
from __future__ import annotations

import argparse
import json
import sys
from typing import Optional


def main(argv: Optional[list] = None) -> int:
    ap = argparse.ArgumentParser(prog="generate", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True)
    ap.add_argument("--ids", action="append", default=[], help="a prompt as comma-separated token ids (repeatable)")
    ap.add_argument("--text", action="append", default=[], help="a prompt as text (needs --tokenizer; repeatable)")
    ap.add_argument("--tokenizer", choices=("llama3", "gpt2"))
    ap.add_argument("--max-new", type=int, default=32)
    ap.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    ap.add_argument("--seed", type=int, default=0)
    ap.add_argument("--dtype", choices=("bfloat16", "float32"))
    ap.add_argument("--max-seqs", type=int, default=8)
    ap.add_argument("--max-model-len", type=int, default=4096)
    ap.add_argument("--device", default="cuda", help="cuda, or cpu for the reference ops")
    a = ap.parse_args(argv)
    if a.text and not a.tokenizer:
        ap.error("--text needs --tokenizer")
    if not a.ids and not a.text:
        ap.error("no prompt: give --ids or --text")
    if a.device == "cuda":
        from .ops.build import ensure_kernels

        ensure_kernels(core="llama" not in a.model.lower())
    import torch

    from .runtime.engine import LLMEngine
    from .runtime.scheduler import TokenScheduler
    from .runtime.weights import load_llm

    tok = None
    if a.tokenizer:
        from .tokenizer import load_tokenizer

        tok = load_tokenizer(a.tokenizer)
    prompts = [[int(t) for t in s.split(",")] for s in a.ids] + [tok.encode(t) for t in a.text]
    model = load_llm(a.model, device=a.device, seed=a.seed, dtype=getattr(torch, a.dtype) if a.dtype else None)
    V = model.cfg.vocab_size
    if any(not 0 <= t < V for p in prompts for t in p):
        ap.error(f"token ids must be below the vocabulary size {V}")
    eng = LLMEngine(model, max_seqs=a.max_seqs, max_model_len=a.max_model_len)
    sched = TokenScheduler(eng, temperature=a.temperature, seed=a.seed)
    for p, out in zip(prompts, sched.generate(prompts, a.max_new, stop_ids=model.cfg.eos_ids)):
        rec = {"prompt_tokens": len(p), "tokens": out}
        if tok is not None:
            rec["text"] = tok.decode(out)
        print(json.dumps(rec), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
