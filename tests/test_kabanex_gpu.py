"""Kabanex on the GPU: every kernel of the layer-stack family alone, then the model through the engine
(step graphs, ragged prompt forwards, cache pages and state slots, scheduler), against the plain
float64 implementation of kabanex_oracle.py."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import kabanex_oracle as O
from voice_enabled_browser_automation_amd import ops
from voice_enabled_browser_automation_amd.models.config import KabanexConfig
from voice_enabled_browser_automation_amd.models.kabanex import KabanexModel
from voice_enabled_browser_automation_amd.runtime.engine import LLMEngine
from voice_enabled_browser_automation_amd.runtime.scheduler import TokenScheduler

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]
BF16, F32 = torch.bfloat16, torch.float32


def rnd(*shape, seed=0, std=1.0, dtype=F32):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * std).to(dtype)


def rel(got, want):
    return float((got.double().cpu() - want.double()).abs().max() / want.double().abs().max().clamp_min(1e-30))


# ----------------------------------------------------------------------------- rows, norms, projections
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,Dp,rows", [(72, 128, 5), (256, 256, 1), (1030, 1152, 33), (4100, 4224, 3), (8192, 8192, 2)])
def test_layernorm_f32(dtype, D, Dp, rows):
    x = rnd(rows, Dp, seed=1, std=3.0) + 20.0    # a mean far from zero: the variance needs the deviations
    w, b = 1 + rnd(D, seed=2, std=0.3), rnd(D, seed=3)
    out = torch.full((rows, Dp), 7.0, dtype=dtype, device=DEV)
    ops.layernorm_f32(x.to(DEV), w.to(DEV), b.to(DEV), eps=1e-3, out=out)
    want = O.layer_norm(x[:, :D].double(), w.double(), b.double(), 1e-3)
    assert rel(out[:, :D], want) < (2e-6 if dtype == F32 else 8e-3)
    assert out[:, D:].abs().sum() == 0


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_f32(dtype):
    t = rnd(50, 72, dtype=dtype)
    ids = torch.tensor([3, 49, 0, 3], dtype=torch.int32)
    out = torch.full((4, 128), 7.0, device=DEV)
    ops.embedding_f32(ids.to(DEV), t.to(DEV), out=out)
    assert torch.equal(out[:, :72].cpu(), t[ids.long()].float()) and out[:, 72:].abs().sum() == 0


@pytest.mark.parametrize("M", [1, 3, 16, 17, 40, 64, 130, 300])
@pytest.mark.parametrize("N,K,ns", [(272, 128, 96), (1040, 384, 640), (4096, 1024, 2048)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_linear_split_and_f32_residual(dtype, M, N, K, ns):
    x, w = rnd(M, K, seed=1, dtype=dtype), rnd(N, K, seed=2, std=K ** -0.5, dtype=dtype)
    y = x.double() @ w.double().T
    tol = 3e-6 if dtype == F32 else 8e-3
    wd = ops.TiledWeight(w.to(DEV)) if dtype == BF16 else w.to(DEV)
    out = torch.zeros(M, ns, dtype=dtype, device=DEV)
    wide = torch.zeros(M, N - ns + 64, dtype=dtype, device=DEV)
    ops.linear_split(x.to(DEV), wd, out, wide[:, 32 : 32 + N - ns])
    assert rel(out, y[:, :ns]) < tol
    assert rel(wide[:, 32 : 32 + N - ns], y[:, ns:].clamp_min(0) ** 2) < 2 * tol
    assert wide[:, :32].abs().sum() == 0 and wide[:, 32 + N - ns :].abs().sum() == 0
    # residual stream: small terms onto large rows must not be rounded to 16 bits
    r = rnd(M, N + 16, seed=3, std=300.0)
    rd = r.to(DEV)
    ops.linear(x.to(DEV), wd, out=rd[:, :N], residual=rd[:, :N])
    assert float((rd[:, :N].cpu().double() - r[:, :N].double() - y).abs().max()) < (1e-3 if dtype == F32 else 2e-3)
    assert torch.equal(rd[:, N:].cpu(), r[:, N:])


# ----------------------------------------------------------------------------- cache + rotation
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dk,dv,rot", [(6, 2, 32, 48, 12), (4, 4, 64, 16, 64), (3, 1, 128, 112, 32)])
def test_qkv_cache_write(dtype, H, G, dk, dv, rot):
    M, bs, nb = 37, 16, 6
    x = rnd(M, H * dk + G * (dk + dv) + 16, seed=1, dtype=dtype)
    pos = torch.arange(M, dtype=torch.int32) + 900
    slots = torch.randperm(nb * bs, generator=torch.Generator().manual_seed(0))[:M]
    slots[5] = -1
    k = torch.zeros(nb, G, bs, dk, dtype=dtype, device=DEV)
    v = torch.zeros(nb, G, dv, bs, dtype=dtype, device=DEV)
    q = torch.zeros(M, H * dk, dtype=dtype, device=DEV)
    rope = ops.rope_table(1000, rot, 250.0, device=DEV)
    ops.qkv_cache_write(x.to(DEV), n_q_heads=H, rot_dims=rot, rope=rope, positions=pos.to(DEV), slots=slots.to(DEV), q_out=q,
                        k_cache=k, v_cache=v)
    xd = x.double()
    wq = O.rotate(xd[:, : H * dk].view(M, H, dk), 250.0, rot, first=900)
    wk = O.rotate(xd[:, H * dk : (H + G) * dk].view(M, G, dk), 250.0, rot, first=900)
    wv = xd[:, (H + G) * dk : (H + G) * dk + G * dv].view(M, G, dv)
    tol = 1e-6 if dtype == F32 else 5e-3
    assert rel(q.view(M, H, dk), wq) < tol
    for m in range(M):
        s = int(slots[m])
        if s >= 0:
            assert rel(k[s // bs, :, s % bs], wk[m]) < 2 * tol and rel(v[s // bs, :, :, s % bs], wv[m]) < 2 * tol
    assert int((k != 0).any(-1).sum()) == G * (M - 1)  # the inert row wrote nothing


# ----------------------------------------------------------------------------- attention
def paged(kn, vn, perm, bs, dtype, extra=3):
    """Natural keys / values [n, G, d] -> caches with the sequence's blocks at perm; other blocks hold rubbish."""
    n, G, dk = kn.shape
    dv = vn.shape[2]
    nb = len(perm) + extra
    k = rnd(nb, G, bs, dk, seed=77, std=30.0, dtype=dtype)
    v = rnd(nb, G, dv, bs, seed=78, std=30.0, dtype=dtype)
    for j in range(n):
        k[perm[j // bs], :, j % bs] = kn[j]
        v[perm[j // bs], :, :, j % bs] = vn[j]
    return k.to(DEV), v.to(DEV)


ATT = [  # H, G, dk, dv, window, keep, bs, n
    (6, 2, 32, 48, 19, 3, 16, 130),
    (4, 4, 64, 16, 64, 0, 16, 200),
    (5, 1, 96, 208, 40, 17, 32, 150),
    (16, 4, 128, 128, 150, 5, 16, 420),
    (8, 8, 64, 80, 16, 16, 16, 90),
    (2, 2, 32, 32, 1000, 4, 16, 100),
    (1, 1, 160, 144, 33, 1, 16, 120),
    (32, 4, 64, 64, 70, 6, 16, 140),
    (20, 1, 32, 32, 30, 2, 16, 90),       # more query heads per kv head than MFMA columns
    (3, 3, 256, 256, 1, 2, 16, 50),       # a window of one
]


def pads(n):
    return 1 << (n - 1).bit_length()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mixed", [True, False])
@pytest.mark.parametrize("case", ATT, ids=[str(c) for c in ATT])
def test_talk_attention(dtype, mixed, case):
    """Rows form and prefill form over one sequence in scattered blocks.  Some keys stand out (their score
    is far above the others'), at block and tile borders and around the kept ones, so every row just inside
    or just outside of an edge changes visibly if the edge is one off."""
    H, G, dk, dv, window, keep, bs, n = case
    gen = torch.Generator().manual_seed(3)
    u = torch.zeros(dk)
    u[0] = 1.0
    q = rnd(n, H, dk, seed=1, std=0.3) + 2.0 * u
    k = rnd(n, G, dk, seed=2, std=0.3)
    for j in {0, keep - 1, keep, keep + 1, 15, 16, 31, 32, 33, n // 2, n - 20}:
        if 0 <= j < n:
            k[j] += (3.0 + float(torch.rand(1, generator=gen))) * u
    v = rnd(n, G, dv, seed=4)
    q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
    T = (torch.eye(H) + rnd(H, H, seed=5, std=0.4)).to(BF16).float() if mixed else torch.eye(H)
    gate = rnd(n, H + 8, seed=6, dtype=dtype)
    scale = 0.7
    m = O.mask(n, window, keep)
    w = O.talk(O.softmax_weights(q.double(), k.double(), scale, m), T.double())
    want = torch.stack([0.8 * torch.sigmoid(gate[:, h : h + 1].double()) * (w[h] @ v[:, h // (H // G)].double())
                        for h in range(H)], 1).reshape(n, H * dv)
    perm = torch.randperm(-(-n // bs) + 3, generator=gen)[: -(-n // bs)].tolist()
    kc, vc = paged(k, v, perm, bs, dtype)
    table = torch.zeros(4, len(perm) + 2, dtype=torch.int32)
    table[2, : len(perm)] = torch.tensor(perm)
    table, qd = table.to(DEV), q.reshape(n, H * dk).to(DEV)
    max_ctx = len(perm) * bs
    sc = ops.TalkScratch([(H, G, dv, window, keep)], max_ctx, DEV)
    kw = dict(n_q_heads=H, scale=scale, window=window, keep=keep, talk=T.to(DEV) if mixed else None,
              talk_frag=ops.talk_fragment(T, G).to(DEV) if pads(G) * pads(H // G) <= 32 else None, out_scale=0.8, max_ctx=max_ctx, scratch=sc)
    pos = torch.arange(n, dtype=torch.int32, device=DEV)
    sid = torch.full((n,), 2, dtype=torch.int32, device=DEV)
    slots = torch.zeros(n, dtype=torch.int64, device=DEV)
    tol = 5e-6 if dtype == F32 else 1.5e-2

    def run(sel, plan):
        sel = torch.tensor(sel, device=DEV)
        out = torch.full((len(sel), H * dv), float("nan"), dtype=dtype, device=DEV)
        ops.talk_attention(qd[sel], kc, vc, table, pos[sel], sid[sel], slots[sel], gate=gate.to(DEV)[sel], out=out, plan=plan, **kw)
        return out

    assert rel(run(list(range(n)), None), want) < tol
    # whole prompt, odd starts, runs of two, single rows beside runs
    for cuts in ([(0, n)], [(7, 2), (30, n - 35), (3, 1), (n - 1, 1), (16, 17)]):
        sel, runs = [], []
        for a, c in cuts:
            c = min(c, n - a)
            runs.append((len(sel), c))
            sel += list(range(a, a + c))
        got = run(sel, ops.plan_runs(runs, DEV, n - 1))
        assert rel(got, want[sel]) < tol
    # inert rows of a padded step are zero and touch nothing
    slots[5] = -1
    got = run(list(range(12)), None)
    assert got[5].abs().sum() == 0 and rel(got[:5], want[:5]) < tol
    assert sc.counters.abs().sum() == 0


def test_prefill_form_takes_the_usual_sizes():
    part = ops.ext().talk_prefill_part
    for H, G, dk, dv in [(4, 2, 64, 128), (16, 4, 128, 128), (32, 8, 128, 128), (6, 2, 96, 192), (8, 1, 256, 64), (12, 12, 64, 64)]:
        assert part(H, G, dk, dv) > 0
    assert part(40, 1, 64, 64) < 0


def test_attention_with_every_key_visible():
    """window 0: ordinary causal attention."""
    H, G, dk, dv, n = 4, 2, 64, 64, 100
    q, k, v = (rnd(n, x, 64, seed=i, dtype=BF16) for i, x in enumerate((H, G, G)))
    w = O.softmax_weights(q.double(), k.double(), 0.125, torch.ones(n, n).tril().bool())
    want = torch.stack([w[h] @ v[:, h // 2].double() for h in range(H)], 1).reshape(n, -1)
    perm = list(range(7))
    kc, vc = paged(k, v, perm, 16, BF16)
    table = torch.tensor([perm], dtype=torch.int32, device=DEV)
    pos = torch.arange(n, dtype=torch.int32, device=DEV)
    for plan in (None, ops.plan_runs([(0, n)], DEV, n - 1)):
        out = torch.zeros(n, H * dv, dtype=BF16, device=DEV)
        ops.talk_attention(q.reshape(n, -1).to(DEV), kc, vc, table, pos, torch.zeros_like(pos), pos.long(), n_q_heads=H,
                           scale=0.125, window=0, keep=0, talk=None, talk_frag=ops.talk_fragment(torch.eye(H), G).to(DEV), gate=None,
                           out_scale=1.0, max_ctx=112, scratch=ops.TalkScratch([(H, G, dv, 0, 0)], 112, DEV), out=out, plan=plan)
        assert rel(out, want) < 1.5e-2


# ----------------------------------------------------------------------------- recurrence
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [24, 256, 700])
def test_mingru(dtype, W):
    """Rows form and scan form over several runs, continuing and fresh, slow and fast channels."""
    tot, R = 0, []
    for sid, pos0, n in ((2, 0, 1), (0, 5, 33), (3, 0, 64), (1, 100, 2), (4, 1, 95)):
        R.append((sid, pos0, n, tot))
        tot += n
    z, x, g = rnd(tot, W, seed=1, std=2, dtype=dtype), rnd(tot, W, seed=2, dtype=dtype), rnd(tot, W, seed=3, dtype=dtype)
    zb, xb = rnd(W, seed=4, std=3.0), rnd(W, seed=5)
    st0 = rnd(5, W, seed=6, std=5.0)
    want, end = torch.zeros(tot, W, dtype=torch.float64), st0.double().clone()
    for sid, p0, n, r0 in R:
        S = O.min_gru(z[r0 : r0 + n].double() + zb.double(), x[r0 : r0 + n].double() + xb.double(), st0[sid].double() if p0 else None)
        want[r0 : r0 + n], end[sid] = S * O.silu(g[r0 : r0 + n].double()) * 0.7, S[-1]
    y = torch.cat([z, x, g], 1).to(DEV)
    ids = torch.cat([torch.full((n,), s) for s, _, n, _ in R]).int().to(DEV)
    pos = torch.cat([torch.arange(p, p + n) for _, p, n, _ in R]).int().to(DEV)
    for plan in (None, ops.plan_runs([(r0, n) for _, _, n, r0 in R], DEV, 200)):
        st = st0.clone().to(DEV)
        out = torch.zeros(tot, W + 8, dtype=dtype, device=DEV)
        ops.mingru(y[:, :W], y[:, W : 2 * W], y[:, 2 * W :], zb.to(DEV), xb.to(DEV), seq_ids=ids, positions=pos,
                   slots=pos.long(), state=st, out_scale=0.7, out=out[:, :W], plan=plan)
        assert rel(out[:, :W], want) < (1e-5 if dtype == F32 else 8e-3)
        assert rel(st, end) < 1e-5 and out[:, W:].abs().sum() == 0


# ----------------------------------------------------------------------------- the model through the engine
CFGS = {
    "odd": O.model_config(72, 101, [
        O.layer_config(6, 2, 20, 24, 12, 19, 3, 40, 56),
        O.layer_config(3, 3, 32, 16, 32, 33, 0, 24, 0, base=5000.0, scale=0.3, ls=1.1, rs=0.4),
        O.layer_config(4, 1, 48, 40, 16, 16, 17, 64, 88)], eps=1e-3),
    "even": O.model_config(384, 512, [
        O.layer_config(8, 4, 64, 64, 32, 48, 4, 256, 512),
        O.layer_config(8, 2, 128, 80, 64, 100, 1, 384, 768, base=1e6)]),
    "one": O.model_config(130, 77, [O.layer_config(1, 1, 32, 16, 2, 5, 1, 1, 33, ls=1.0, rs=1.0)]),
}
LIMIT = {F32: 2e-5, BF16: 3e-2}


def tokens(n, seed, vocab):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


_MODELS = {}


def setup(name, dtype, **kw):
    if (name, dtype) not in _MODELS:
        w = O.random_weights(CFGS[name], 5)
        _MODELS[name, dtype] = (w, KabanexModel(KabanexConfig.from_json(CFGS[name]), weights=w, device=DEV, dtype=dtype))
    w, m = _MODELS[name, dtype]
    return CFGS[name], w, LLMEngine(m, **dict(dict(max_seqs=4, max_model_len=512), **kw))


_WANT = {}


def oracle(name, n, seed):
    key = (name, n, seed)
    if key not in _WANT:
        t = tokens(n, seed, CFGS[name]["vocab"])
        _WANT[key] = (t, O.forward(CFGS[name], O.random_weights(CFGS[name], 5), t))
    return _WANT[key]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CFGS))
def test_residual_after_every_layer(name, dtype):
    cfg, w, eng = setup(name, dtype)
    t = tokens(50, 9, cfg["vocab"])
    _, res = O.forward(cfg, w, t, layers=True)
    m, seen = eng.model, []
    use_graphs, eng.use_graphs = eng.use_graphs, False
    run = m._layer
    m._layer = lambda li, bufs, M, kv, x, *a: (run(li, bufs, M, kv, x, *a), seen.append(x[:50, : cfg["width"]].clone()))
    try:
        eng.step_batch([(eng.new_sequence([]), t)], [49])
    finally:
        del m._layer
        eng.use_graphs = use_graphs
    assert len(seen) == len(res)
    for g, r in zip(seen, res):
        assert rel(g, r) < (1e-5 if dtype == F32 else 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CFGS))
@pytest.mark.parametrize("cuts", [[150], [2], [16, 1], [70, 3, 2], [1], [100, 50]], ids=str)
def test_prompts_in_portions(name, dtype, cuts):
    cfg, w, eng = setup(name, dtype)
    t, want = oracle(name, 150, 1)
    seq, out, i, k = eng.new_sequence([]), [], 0, 0
    while i < len(t):
        part = t[i : i + cuts[k % len(cuts)]]
        out.append(eng.step_batch([(seq, part)], range(len(part))).clone())
        i, k = i + len(part), k + 1
    assert O.logit_error(torch.cat(out), want).max() < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["odd", "even"])
@pytest.mark.parametrize("big", [False, True])
def test_mixed_batches_with_reused_pages_and_slots(name, dtype, big):
    """Unequal requests in common steps, portions beside single tokens, requests left out of a step, pages
    and slots used again -- against each request alone.  big: steps past the step graphs' rows."""
    lens = (230, 41, 7, 64, 150, 1, 90, 33)
    need = sorted((-(-n // 64) * 4 for n in lens), reverse=True)
    cfg, w, eng = setup(name, dtype, max_seqs=3, kv_blocks=1 + sum(need[:3]))
    reqs = {n: oracle(name, n, 100 + n) for n in lens}
    live, queue, at, got, rng = {}, list(lens), {}, {n: [] for n in lens}, np.random.default_rng(1)
    sids = []
    while queue or live:
        while queue and len(live) < 3:
            n = queue.pop(0)
            live[n], at[n] = eng.new_sequence([]), 0
            sids.append(live[n].sid)
        entries = []
        for n in live:
            if len(live) > 1 and rng.random() < 0.2:
                continue
            k = int(rng.choice([1, 2, 30, 64, 100] if big else [1, 1, 2, 5, 17]))
            entries.append((n, reqs[n][0][at[n] : at[n] + k]))
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
    assert len(sids) == len(lens) and len(set(sids)) == 3
    for n in lens:
        assert O.logit_error(torch.cat(got[n]), reqs[n][1]).max() < LIMIT[dtype], n


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    """Decoding far past every window, through the captured step graph, its first replay included (the
    capture's warm-up forwards must not advance the recurrent state)."""
    t, want = oracle("even", 260, 4)
    cfg, w, eng = setup("even", dtype)
    seq = eng.new_sequence([])
    out = [eng.step_batch([(seq, t[:5])], range(5)).clone()]
    for i in range(5, 260):
        out.append(eng.step_batch([(seq, t[i : i + 1])], [0]).clone())
    assert eng.stats["graph_replays"] >= 250
    assert O.logit_error(torch.cat(out), want).max() < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_match_eager_steps(dtype):
    """Every replay of the step graphs against the same step run eagerly, other work in between."""
    cfg, w, ga = setup("odd", dtype)
    _, _, eb = setup("odd", dtype, use_graphs=False)
    seqs = [(ga.new_sequence([]), eb.new_sequence([])) for _ in range(3)]
    for step in range(12):
        batch = [(p, tokens(1 + (step + i) % 3, 10 * step + i, 101)) for i, p in enumerate(seqs) if (step + i) % 4]
        n = sum(len(t) for _, t in batch)
        a = ga.step_batch([(p[0], t) for p, t in batch], range(n)).clone()
        torch.cuda.synchronize()
        junk = torch.randn(256, 256, device=DEV).sum()  # noqa: F841
        b = eb.step_batch([(p[1], t) for p, t in batch], range(n)).clone()
        assert torch.equal(a, b), step
        for x, y in zip(ga.kv.state, eb.kv.state):
            assert torch.equal(x[:3], y[:3])


def test_far_keys_and_edges_in_decoding():
    """A prompt longer than the window with kept first tokens: decoded logits depend on the first tokens
    and on the last one inside the window, and not on the one just outside (no other layer carries it)."""
    cfg = O.model_config(128, 64, [O.layer_config(4, 2, 32, 32, 16, 40, 3, 16, 64)])
    w = O.random_weights(cfg, 8)
    for k in ("l0.mix.right.o",):
        w[k] = torch.zeros_like(w[k])    # the recurrence reaches past every window: taken out here
    m = KabanexModel(KabanexConfig.from_json(cfg), weights=w, device=DEV, dtype=F32)
    eng = LLMEngine(m, max_seqs=2, max_model_len=256)
    t = tokens(101, 3, 64)

    def last(tt, cut):
        s = eng.new_sequence([])
        if cut:
            eng.step_batch([(s, tt[:cut])])
            for x in tt[cut:-1]:
                eng.step_batch([(s, [x])])
            r = eng.step_batch([(s, tt[-1:])], [0]).clone()
        else:
            r = eng.step_batch([(s, tt)], [len(tt) - 1]).clone()
        eng.free_sequence(s)
        return r

    for cut in (0, 70):
        base = last(t, cut)
        for j, seen in ((0, True), (2, True), (3, False), (100 - 39, True), (100 - 40, False), (50, False)):
            tt = list(t)
            tt[j] = (tt[j] + 1) % 64
            d = float((last(tt, cut) - base).abs().max())
            assert (d > 1e-4) if seen else (d == 0), (cut, j, d)


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_scheduler(dtype):
    cfg, w, eng = setup("even", dtype, max_seqs=2)
    prompts = [tokens(n, 40 + n, 512) for n in (37, 3, 90)]
    outs = TokenScheduler(eng, token_budget=80).generate(prompts, 8)
    for p, o in zip(prompts, outs):
        want = O.forward(cfg, w, p + o)
        for i, tok in enumerate(o):  # (each token is the oracle's choice given the tokens before it, up to near-ties)
            row = want[len(p) - 1 + i]
            assert row.max() - row[tok] < (1e-4 if dtype == F32 else 0.08) * row.std(), (i, tok)


def test_sampling_at_a_temperature_is_reproducible():
    _, _, eng = setup("even", BF16, max_seqs=2)
    p = tokens(20, 1, 512)
    a, b = (TokenScheduler(eng, temperature=1.5, seed=s).generate([p], 12)[0] for s in (3, 3))
    c = TokenScheduler(eng, temperature=1.5, seed=4).generate([p], 12)[0]
    assert a == b and a != c


def test_trace_replay_command(tmp_path):
    cfg = CFGS["odd"]
    w = O.random_weights(cfg, 5)
    O.save_model(str(tmp_path / "m"), cfg, w)
    t, want = oracle("odd", 150, 1)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:100], "want": [99, 7]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t[100:], "want": [49]}, {"id": "b", "tokens": t[:2], "want": [1]}],
              "end": ["a", "b"]}]
    for dtype, lim in (("bfloat16", LIMIT[BF16]), ("float32", LIMIT[F32])):
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype, "--out",
                            str(tmp_path / dtype), "--max-tokens", "256"], input="".join(json.dumps(s) + "\n" for s in steps),
                           capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [x for x in r.stdout.split("\n") if x.startswith("done")] == ["done 0", "done 1"]
        got = torch.cat([torch.from_numpy(np.fromfile(tmp_path / dtype / f"{i}.f32", dtype="<f4")).view(-1, 101) for i in (0, 1)])
        assert O.logit_error(got, want[[99, 7, 149, 1]]).max() < lim


def test_intent_engine_serves_a_kabanex_preset():
    from voice_enabled_browser_automation_amd.brain.intent_engine import LLMIntentEngine
    from voice_enabled_browser_automation_amd.contracts import ParseResponse, safe_parse
    from voice_enabled_browser_automation_amd.runtime.weights import load_llm
    from voice_enabled_browser_automation_amd.tokenizer import load_tokenizer

    eng = LLMEngine(load_llm("kabanex-tiny", device=DEV), max_seqs=4, max_model_len=2048)
    brain = LLMIntentEngine(eng, load_tokenizer("llama3"), budget_chars=200, temperature=0.0)
    reqs = [{"text": s, "context": {}} for s in ("scroll down", "search wireless earbuds", "go back")]
    outs = brain.parse_many(reqs)
    assert all(safe_parse(ParseResponse, o).success for o in outs)


def test_native_path_only():
    """Nothing of the model leaves the hand-written kernels (strict native mode would raise)."""
    _, _, eng = setup("even", BF16)
    before = dict(ops.vendor_fallbacks)
    s = eng.new_sequence([])
    eng.step_batch([(s, tokens(150, 2, 512))], [149])
    eng.step_batch([(s, [1])], [0])
    assert ops.vendor_fallbacks == before
