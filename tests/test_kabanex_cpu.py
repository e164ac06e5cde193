"""Kabanex on the CPU reference ops: reading a checkpoint folder, and the engine's, cache's, state
slots' and scheduler's part in it (portions, mixed batches, reuse, generation) against the plain
implementation of kabanex_oracle.py.  The GPU kernels have the same tests in test_kabanex_gpu.py."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import kabanex_oracle as O
from voice_enabled_browser_automation_amd import ops
from voice_enabled_browser_automation_amd.models import model_class
from voice_enabled_browser_automation_amd.models.config import KabanexConfig, config_from_dir, get_config
from voice_enabled_browser_automation_amd.models.kabanex import KabanexModel
from voice_enabled_browser_automation_amd.runtime.engine import LLMEngine
from voice_enabled_browser_automation_amd.runtime.kv_cache import CacheLayer, PagedKVCache
from voice_enabled_browser_automation_amd.runtime.scheduler import TokenScheduler
from voice_enabled_browser_automation_amd.runtime.weights import load_llm

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

# unequal layers: odd sizes, one layer without a feed-forward, windows and kept keys on and off tile borders
CFG = O.model_config(72, 101, [
    O.layer_config(6, 2, 20, 24, 12, 19, 3, 40, 56),
    O.layer_config(3, 3, 32, 16, 32, 33, 0, 24, 0, base=5000.0, scale=0.3, ls=1.1, rs=0.4),
    O.layer_config(4, 1, 48, 40, 16, 16, 17, 64, 88),
], eps=1e-3)


def tokens(n, seed, vocab=101):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


@pytest.fixture(scope="module")
def folder(tmp_path_factory):
    d = str(tmp_path_factory.mktemp("kabanex") / "m")
    O.save_model(d, CFG, O.random_weights(CFG, 5))
    return d


@pytest.fixture(scope="module")
def weights():
    return O.random_weights(CFG, 5)


@pytest.fixture(scope="module")
def model(folder):
    return load_llm(folder, device="cpu", dtype=torch.float32)


def engine(model, **kw):
    return LLMEngine(model, **dict(dict(max_seqs=3, max_model_len=256, kv_blocks=40), **kw))


def test_config_and_registry(folder):
    cfg = config_from_dir(folder)
    assert isinstance(cfg, KabanexConfig) and get_config(folder) == cfg and model_class(cfg) is KabanexModel
    assert cfg.vocab_size == 101 and cfg.hidden == 72 and cfg.n_layers == 3 and cfg.norm_eps == 1e-3
    a = cfg.layers[2].left
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, a.rot_dims) == (4, 1, 48, 40, 16, 17, 16)
    assert cfg.layers[1].ffn == 0 and cfg.layers[1].left.scale == 0.3 and cfg.layers[1].right_scale == 0.4
    assert model_class(get_config("kabanex-tiny")) is KabanexModel


@pytest.mark.parametrize("change", [
    lambda j: j["layers"][0].update(type="series"),
    lambda j: j["layers"][0]["mlp"].update(kind="routed"),
    lambda j: j["layers"][0]["mixer"]["left"].update(kv_heads=4),
    lambda j: j["layers"][0]["mixer"]["left"]["rot"].update(dims=22),
    lambda j: j["layers"][0]["mixer"]["left"]["mask"].update(size=0),
])
def test_config_refuses_what_it_does_not_know(change):
    j = json.loads(json.dumps(CFG))
    change(j)
    with pytest.raises(ValueError):
        KabanexConfig.from_json(j)
    with pytest.raises(KeyError):
        config = json.loads(json.dumps(CFG))
        del config["layers"][0]["mixer"]["left"]["scale"]
        KabanexConfig.from_json(config)


def test_unknown_architecture_is_an_error(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nothing"}))
    with pytest.raises(KeyError):
        config_from_dir(str(tmp_path))


def test_wrong_tensor_shape_is_an_error(weights):
    w = dict(weights)
    w["l0.mix.left.q"] = w["l0.mix.left.q"][:-1]
    with pytest.raises(ValueError):
        KabanexModel(KabanexConfig.from_json(CFG), weights=w, dtype=torch.float32)


def test_whole_prompt_and_layers(model, weights):
    t = tokens(90, 1)
    want, res = O.forward(CFG, weights, t, layers=True)
    eng = engine(model)
    seq = eng.new_sequence([])
    seen = []
    run = model._layer
    model._layer = lambda li, bufs, M, kv, x, *a: (run(li, bufs, M, kv, x, *a), seen.append(x[:, :72].clone()))
    try:
        got = eng.step_batch([(seq, t)], range(len(t)))
    finally:
        del model._layer
    for g, r in zip(seen, res):
        assert torch.allclose(g.double(), r, atol=2e-4)
    assert O.logit_error(got, want).max() < 1e-5


@pytest.mark.parametrize("cuts", [[2], [1], [16], [17, 3], [70, 2]])
def test_portions(model, weights, cuts):
    t = tokens(83, 2)
    want = O.forward(CFG, weights, t)
    eng = engine(model)
    seq, out, i, k = eng.new_sequence([]), [], 0, 0
    while i < len(t):
        part = t[i : i + cuts[k % len(cuts)]]
        out.append(eng.step_batch([(seq, part)], range(len(part))).clone())
        i, k = i + len(part), k + 1
    assert O.logit_error(torch.cat(out), want).max() < 1e-5


def test_mixed_batches_and_reuse(model, weights):
    """Unequal requests in common steps (one skipping steps), pages and slots given back and used again,
    against every request alone; the pool is exactly as large as the live requests need."""
    eng = engine(model, kv_blocks=1 + 3 * 6)
    reqs = {n: tokens(n, n) for n in (95, 41, 7, 64, 88, 1)}
    want = {n: O.forward(CFG, weights, t) for n, t in reqs.items()}
    live, queue, at, got, rng = {}, list(reqs), {}, {n: [] for n in reqs}, np.random.default_rng(0)
    used_sids = []
    while queue or live:
        while queue and len(live) < 3:
            n = queue.pop(0)
            live[n], at[n] = eng.new_sequence([]), 0
            used_sids.append(live[n].sid)
        entries = []
        for n, seq in live.items():
            if rng.random() < 0.25 and len(live) > 1:
                continue
            k = int(rng.choice([1, 1, 2, 5, 17, 40]))
            entries.append((n, reqs[n][at[n] : at[n] + k]))
        if not entries:
            continue
        lg = eng.step_batch([(live[n], p) for n, p in entries], range(sum(len(p) for _, p in entries)))
        i = 0
        for n, p in entries:
            got[n].append(lg[i : i + len(p)].clone())
            i += len(p)
            at[n] += len(p)
        for n in [n for n, _ in entries if at[n] == n]:
            eng.free_sequence(live.pop(n))
    assert len(set(used_sids)) == 3 and len(used_sids) == 6
    for n in reqs:
        assert O.logit_error(torch.cat(got[n]), want[n]).max() < 1e-5, n
    assert eng.blocks.n_free() == 18


def test_one_planted_mistake_per_mechanism_shows(weights):
    """The comparisons are sharp: the oracle with one mechanism slightly wrong differs by far more than
    the tolerance used above."""
    t = tokens(60, 3)
    want = O.forward(CFG, weights, t)
    j = lambda: json.loads(json.dumps(CFG))  # noqa: E731

    def left(f):
        c = j()
        for L in c["layers"]:
            f(L["mixer"]["left"])
        return c, weights

    one_off = left(lambda a: a["mask"].update(size=a["mask"]["size"] + 1))
    no_sink = left(lambda a: a["mask"].update(keep_first=0))
    sink_off = left(lambda a: a["mask"].update(keep_first=a["mask"]["keep_first"] + 1))
    rot = left(lambda a: a["rot"].update(dims=a["rot"]["dims"] - 2))
    untalked = CFG, {k: (torch.eye(v.shape[0]) if k.endswith("talk") else v) for k, v in weights.items()}
    for cfg, w in (one_off, no_sink, sink_off, rot, untalked):
        assert O.logit_error(O.forward(cfg, w, t), want).max() > 1e-3


def test_state_starts_from_zero_in_a_used_slot(model, weights):
    eng = engine(model, max_seqs=1)
    for seed in (11, 12):
        t = tokens(30, seed)
        seq = eng.new_sequence([])
        got = eng.step_batch([(seq, t)], range(len(t)))
        assert O.logit_error(got, O.forward(CFG, weights, t)).max() < 1e-5
        eng.free_sequence(seq)
    assert all(s.abs().max() > 0 for s in eng.kv.state)


def test_no_prefix_cache_for_a_recurrent_model(model):
    """Blocks alone cannot resume a sequence: its state would be missing."""
    eng = engine(model)
    t = tokens(64, 4)
    for _ in range(2):
        seq = eng.new_sequence(t)
        assert seq.n_computed == 0
        eng.prefill(seq)
        eng.free_sequence(seq)
    assert eng.blocks.n_free() == eng.blocks.num_blocks - 1 and not eng.blocks.cache


def test_engine_prefill_paths_agree(model, weights):
    t = tokens(150, 6)
    want = O.forward(CFG, weights, t)
    eng = engine(model)
    a, b = eng.new_sequence(t), eng.new_sequence(t)
    assert O.logit_error(eng.prefill(a, chunk=100), want[-1:]).max() < 1e-5
    eng.prefill_batch([(b, len(t) - 1)])
    got = eng.run_rows([(b, t[-1])])
    assert O.logit_error(got, want[-1:]).max() < 1e-5


def greedy(cfg, weights, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(O.forward(cfg, weights, t)[-1].argmax()))
    return t[len(prompt):]


def test_greedy_generation_through_the_scheduler(model, weights):
    prompts = [tokens(n, 20 + n) for n in (37, 3, 70, 1, 18)]
    eng = engine(model, max_seqs=2)
    sched = TokenScheduler(eng, token_budget=24)
    outs = sched.generate(prompts, 6)
    assert outs == [greedy(CFG, weights, p, 6) for p in prompts]
    assert sched.stats["rows"] == sum(len(p) + 5 for p in prompts)
    # a stop token ends a request
    assert sched.generate([prompts[0]], 6, stop_ids=[outs[0][1]])[0] == outs[0][: outs[0].index(outs[0][1]) + 1]


def test_scheduler_waits_for_blocks(model):
    eng = engine(model, max_seqs=3, kv_blocks=1 + 5)
    sched = TokenScheduler(eng)
    a = sched.submit(tokens(40, 1), 8)   # 3 blocks
    b = sched.submit(tokens(40, 2), 8)   # 3 blocks: does not fit beside it
    sched.step()
    assert len(sched.active) == 1 and len(sched.waiting) == 1
    sched.run_until_idle()
    assert a.done and b.done and eng.blocks.n_free() == 5
    with pytest.raises(ValueError):
        sched.submit(tokens(90, 3), 8)


@pytest.mark.parametrize("name", ["llama-tiny", "gpt2-tiny"])
def test_scheduler_and_step_batch_serve_the_other_models(name):
    m = load_llm(name, device="cpu", dtype=None)
    eng = LLMEngine(m, max_seqs=2, max_model_len=256)
    t = tokens(90, 8, vocab=1000)
    a = eng.new_sequence([], use_prefix_cache=False)
    whole = eng.step_batch([(a, t)], [0, 50, 89]).clone()
    b, c, got = eng.new_sequence([], use_prefix_cache=False) if eng.free_sids else None, None, []
    for i in range(0, 90, 30):
        lg = eng.step_batch([(b, t[i : i + 30])], [w - i for w in (0, 50, 89) if i <= w < i + 30])
        if lg is not None:
            got.append(lg.clone())
    assert (torch.cat(got) - whole).abs().max() <= 0.02 * whole.abs().max()
    eng.free_sequence(a)
    eng.free_sequence(b)
    outs = TokenScheduler(eng).generate([t[:20], t[:7]], 4)
    assert [len(o) for o in outs] == [4, 4]


def test_cache_with_unequal_layers():
    layers = [CacheLayer(2, 32, 16, True, 24), CacheLayer(1, 64, 48)]
    kv = PagedKVCache.from_layers(layers, 16, 5, 3, dtype=torch.float32)
    assert kv.k[0].shape == (5, 2, 16, 32) and kv.v[0].shape == (5, 2, 16, 16) and kv.state[0].shape == (3, 24)
    assert kv.k[1].shape == (5, 1, 16, 64) and kv.v[1].shape == (5, 1, 16, 48) and kv.state[1].shape == (3, 0)
    assert PagedKVCache.layer_bytes_per_block(layers, 16) == 2 * 16 * (2 * 48 + 112)


@pytest.mark.parametrize("H,G", [(1, 1), (2, 1), (4, 2), (6, 2), (8, 8), (16, 4), (12, 3), (32, 8), (24, 2)])
def test_talk_fragment_is_the_matrix_for_both_halves(H, G):
    """The A operand times (hi | lo) stacked heads is talk @ (hi + lo), in the padded head order."""
    T = torch.randn(H, H).to(torch.bfloat16).float()
    fr = ops.talk_fragment(T, G).float()
    R = H // G
    up = lambda n: 1 << (n - 1).bit_length()  # noqa: E731
    HT = up(G) * up(R)
    A = fr.view(-1, 4, 16, 8).permute(0, 2, 1, 3).reshape(-1, 32)          # [rows, k]
    order = [(h // R) * up(R) + h % R for h in range(H)]
    hi, lo = torch.zeros(max(HT, 4)), torch.zeros(max(HT, 4))
    hi[order], lo[order] = torch.randn(H), torch.randn(H) * 0.01
    if HT == 32:
        got = A @ hi + A @ lo
    else:
        x = torch.zeros(32)
        x[: 2 * max(HT, 4)] = torch.cat([hi, lo])
        got = A @ x
    assert torch.allclose(got[order], T @ (hi + lo)[order], atol=1e-4)


def test_prefill_splits():
    from voice_enabled_browser_automation_amd.ops.stack import prefill_splits

    assert prefill_splits(128, 2047, 1024, 4, 256) == 2 and prefill_splits(300, 5000, 0, 0, 256) == 1
    assert prefill_splits(4, 63, 1024, 0, 256) == 1 and prefill_splits(4, 4095, 1024, 4, 256) == 9


def test_trace_replay_command(folder, weights, tmp_path):
    """bin/trace_run end to end on the reference ops: two requests in common steps, wanted logits in order."""
    a, b = tokens(70, 31), tokens(20, 32)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:69], "want": [0, 68]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[69:], "want": []}, {"id": "b", "tokens": b[:2], "want": []}],
              "end": ["a"]},
             {"step": 2, "entries": [{"id": "b", "tokens": b[2:], "want": [17, 3]}], "end": ["b"]}]
    out = tmp_path / "out"
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128", "--device", "cpu"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=300, env=dict(os.environ, PYTHONDONTWRITEBYTECODE="1"))
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.split("\n") if x] == ["done 0", "done 1", "done 2"]
    wa, wb = O.forward(CFG, weights, a), O.forward(CFG, weights, b)
    read = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4")).view(-1, 101)  # noqa: E731
    assert O.logit_error(read(0), wa[[0, 68]]).max() < 1e-5
    assert not (out / "1.f32").exists()
    assert O.logit_error(read(2), wb[[19, 5]]).max() < 1e-5


def test_generate_command(folder, weights):
    r = subprocess.run([sys.executable, "-m", "voice_enabled_browser_automation_amd.generate", "--model", folder, "--ids",
                        "5,6,7", "--ids", "9", "--max-new", "3", "--dtype", "float32", "--device", "cpu", "--max-model-len",
                        "64"], capture_output=True, text=True, timeout=300, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-2000:]
    got = [json.loads(x)["tokens"] for x in r.stdout.split("\n") if x]
    assert got == [greedy(CFG, weights, p, 3) for p in ([5, 6, 7], [9])]


def test_intent_engine_serves_a_kabanex_preset():
    """The grammar-constrained intent scheduler runs it like its other models."""
    from voice_enabled_browser_automation_amd.brain.intent_engine import LLMIntentEngine
    from voice_enabled_browser_automation_amd.contracts import ParseResponse, safe_parse
    from voice_enabled_browser_automation_amd.tokenizer import load_tokenizer

    m = load_llm("kabanex-tiny", device="cpu")
    eng = LLMEngine(m, max_seqs=2, max_model_len=2048)
    brain = LLMIntentEngine(eng, load_tokenizer("llama3"), budget_chars=160)
    out = brain.parse({"text": "scroll down", "context": {}})
    assert safe_parse(ParseResponse, out).success
