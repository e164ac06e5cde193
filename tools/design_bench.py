"""Prefill and decode throughput of one model design beside the framework's closest model at equal size
(bench.py --design; random weights, a few layers of a real model's sizes).

    python bench.py --design ripupel|kabanex [--design-size s1,s2,s4] [--design-only ripupel|kabanex|llama]

Per size: prompt tokens/s of one 2048-token prompt, and generated tokens/s of 1 / 16 / 64 sequences decoding
at ~1.5k tokens of context through the captured step graphs (LM head included, sampling not).  The two
models are timed in turn, round by round; the median round counts.
"""
from __future__ import annotations

import json
import statistics
import time

import torch

VOCAB = 32768
LAYERS = 8
CLOSEST = {"ripupel": "kabanex", "kabanex": "llama"}  # the model a design is timed beside
PROMPT = 2048
CONTEXT = 1536

# width, heads, kv heads, head size, feed-forward: layers of (nearly) equal bytes.  Ripupel: ``top`` of ``experts``
# feed-forwards of size expert_ff in every second layer, together as wide as the dense one
SIZES = {
    "s1": dict(hidden=1024, heads=8, kv_heads=4, dim=128, ffn=4096, experts=16, top=4, expert_ff=1024),
    "s2": dict(hidden=2048, heads=16, kv_heads=4, dim=128, ffn=8192, experts=16, top=4, expert_ff=2048),
    "s4": dict(hidden=4096, heads=32, kv_heads=8, dim=128, ffn=14336, experts=16, top=4, expert_ff=3584),
}


def build(design: str, size: str, dev):
    from voice_enabled_browser_automation_amd.models.config import LlamaConfig, kabanex_stack, ripupel_stack
    from voice_enabled_browser_automation_amd.models.kabanex import KabanexModel
    from voice_enabled_browser_automation_amd.models.llama import LlamaModel
    from voice_enabled_browser_automation_amd.models.ripupel import RipupelModel

    s = SIZES[size]
    if design == "ripupel":
        return RipupelModel(ripupel_stack(size, vocab=VOCAB, hidden=s["hidden"], n_layers=LAYERS, heads=s["heads"], dim=s["dim"],
                                          rot_dim=64, vdim=s["dim"], kv_rank=512, width=s["hidden"], blocks=s["hidden"] // 256,
                                          ffn=s["ffn"], experts=s["experts"], top=s["top"], expert_ff=s["expert_ff"]),
                            device=dev, seed=1)
    if design == "llama":
        return LlamaModel(LlamaConfig(name=size, vocab_size=VOCAB, hidden=s["hidden"], n_layers=LAYERS, n_heads=s["heads"],
                                      n_kv_heads=s["kv_heads"], head_dim=s["dim"], ffn=s["ffn"]), device=dev, seed=1)
    return KabanexModel(kabanex_stack(size, vocab=VOCAB, hidden=s["hidden"], n_layers=LAYERS, heads=s["heads"],
                                      kv_heads=s["kv_heads"], dim=s["dim"], vdim=s["dim"], window=1024, keep_first=4,
                                      width=s["hidden"], ffn=s["ffn"]), device=dev, seed=1)


class Bed:
    """One model with its engine, ready to time."""

    def __init__(self, design: str, size: str, dev):
        from voice_enabled_browser_automation_amd.runtime.engine import LLMEngine

        self.model = build(design, size, dev)
        self.eng = LLMEngine(self.model, max_seqs=64, max_model_len=PROMPT + 64, kv_blocks=64 * 110 + 1)
        self.gen = torch.Generator().manual_seed(0)

    def ids(self, n):
        return torch.randint(0, VOCAB, (n,), generator=self.gen).tolist()

    def prefill(self, reps: int) -> float:
        """ms per 2048-token prompt."""
        toks, ms = self.ids(PROMPT), []
        for _ in range(reps):
            seq = self.eng.new_sequence(toks, use_prefix_cache=False)
            torch.cuda.synchronize()
            t0 = time.perf_counter()
            self.eng.prefill(seq)
            torch.cuda.synchronize()
            ms.append((time.perf_counter() - t0) * 1e3)
            self.eng.free_sequence(seq, publish=False)
        return statistics.median(ms)

    def fill(self, n: int):
        """n sequences at CONTEXT tokens (random cache contents: only the time matters)."""
        seqs = []
        for _ in range(n):
            s = self.eng.new_sequence([], use_prefix_cache=False)
            s.tokens = self.ids(CONTEXT)
            self.eng._ensure_blocks(s, CONTEXT)
            s.n_computed = CONTEXT
            seqs.append(s)
        return seqs

    def decode(self, n: int, steps: int) -> float:
        """ms per decode step of n sequences."""
        seqs = self.fill(n)
        toks = self.ids(n)

        def step():
            self.eng.run_rows(list(zip(seqs, toks)), check=False)

        for _ in range(3):
            step()
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        for _ in range(steps):
            step()
        torch.cuda.synchronize()
        ms = (time.perf_counter() - t0) * 1e3 / steps
        for s in seqs:
            self.eng.free_sequence(s, publish=False)
        return ms


def run(args) -> None:
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    designs = [args.design_only] if args.design_only else [args.design, CLOSEST[args.design]]
    res = {"metric": "prefill / decode throughput (tokens/s) of a model design beside the closest model at equal size",
           "unit": "tokens/s", "n_gpus": 1, "dtype": "bf16", "data": "random weights, random tokens", "layers": LAYERS,
           "prompt": PROMPT, "context": CONTEXT, "sizes": {}}
    for size in args.design_size.split(","):
        beds = {d: Bed(d, size, dev) for d in designs}
        out = {d: {"layer_mb": round((b.model.weight_bytes() - b.model.lm_head.numel() * 2) / LAYERS / 1e6, 1)}
               for d, b in beds.items()}
        for d, b in beds.items():
            b.prefill(2)
        pre = {d: [] for d in beds}
        dec = {d: {n: [] for n in (1, 16, 64)} for d in beds}
        for _ in range(args.design_rounds):
            for d, b in beds.items():
                pre[d].append(b.prefill(5))
                for n in (1, 16, 64):
                    dec[d][n].append(b.decode(n, 30))
        for d in beds:
            ms = statistics.median(pre[d])
            out[d]["prefill_ms"], out[d]["prefill_tok_s"] = round(ms, 3), round(PROMPT / ms * 1e3)
            for n in (1, 16, 64):
                ms = statistics.median(dec[d][n])
                out[d][f"decode{n}_ms"], out[d][f"decode{n}_tok_s"] = round(ms, 4), round(n / ms * 1e3)
        res["sizes"][size] = out
        print(json.dumps({size: out}), flush=True)
        del beds
        torch.cuda.empty_cache()
    first = res["sizes"][args.design_size.split(",")[0]]
    res["value"] = first[designs[0]]["prefill_tok_s"]
    print(json.dumps(res), flush=True)
