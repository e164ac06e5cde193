"""Ripupel on the GPU: every kernel of its mixers and feed-forwards alone, then the model through the
engine (step graphs, ragged prompt forwards, cache pages and state slots, scheduler), against the plain
float64 implementation of ripupel_oracle.py."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import ripupel_oracle as O
from voice_enabled_browser_automation_amd import ops
from voice_enabled_browser_automation_amd.models.config import RipupelConfig
from voice_enabled_browser_automation_amd.models.ripupel import RipupelModel
from voice_enabled_browser_automation_amd.ops import mixers
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


def up(n, m):
    return -(-n // m) * m


# ----------------------------------------------------------------------------- norms, embedding, dense ff
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,rows,parts", [(72, 5, 1), (75, 3, 4), (256, 1, 2), (1030, 33, 1), (2048, 7, 3), (4100, 3, 1), (8192, 2, 2)])
def test_add_norm(dtype, D, rows, parts):
    Dp = up(D, 128)
    x = rnd(rows, Dp, seed=1, std=3.0) + 20.0        # means far from zero: the variances need the deviations
    br = (rnd(rows * parts, up(D, 16), seed=2) - 5.0).to(dtype)
    x[:, D:], br[:, D:] = 0, 7.0                     # (what lies in padding columns does not count)
    w1, w2 = 1 + rnd(D, seed=3, std=0.3), 1 + rnd(D, seed=4, std=0.3)
    y = br[:, :D].double().view(rows, parts, D).sum(1)
    want = x[:, :D].double() + O.layer_norm(y, w1.double(), 1e-3)
    h = torch.full((rows, Dp), 7.0, dtype=dtype, device=DEV)
    for nxt in (w2, None):
        xd = x.to(DEV)
        ops.add_norm(xd, br.to(DEV), w1.to(DEV), None if nxt is None else nxt.to(DEV), eps=1e-3, out=h, n_parts=parts)
        assert rel(xd[:, :D], want) < 2e-6 and xd[:, D:].abs().sum() == 0
    hw = O.layer_norm(want, w2.double(), 1e-3)
    assert rel(h[:, :D], hw) < (4e-6 if dtype == F32 else 8e-3) and h[:, D:].abs().sum() == 0


@pytest.mark.parametrize("dtype", DTYPES)
def test_norm_without_bias_and_scaled_embedding(dtype):
    x, w = rnd(3, 256, seed=1) + 4, rnd(200, seed=2)
    out = torch.full((3, 256), 7.0, dtype=dtype, device=DEV)
    ops.layernorm_f32(x.to(DEV), w.to(DEV), None, eps=1e-3, out=out)
    assert rel(out[:, :200], O.layer_norm(x[:, :200].double(), w.double(), 1e-3)) < (2e-6 if dtype == F32 else 8e-3)
    t = rnd(50, 72, dtype=dtype)
    ids = torch.tensor([3, 49, 0], dtype=torch.int32)
    e = torch.full((3, 128), 7.0, device=DEV)
    ops.embedding_f32(ids.to(DEV), t.to(DEV), out=e, scale=0.3)
    assert torch.allclose(e[:, :72].cpu(), t[ids.long()].float() * 0.3) and e[:, 72:].abs().sum() == 0


@pytest.mark.parametrize("M,N,K", [(1, 64, 128), (5, 160, 96), (70, 256, 384), (200, 2048, 512)])
def test_linear_swiglu_in_32_bit(M, N, K):
    x, g, u = rnd(M, K, seed=1), rnd(N // 2, K, seed=2, std=K ** -0.5), rnd(N // 2, K, seed=3, std=K ** -0.5)
    out = torch.zeros(M, N // 2 + 16, device=DEV)
    ops.linear_swiglu(x.to(DEV), ops.interleave_gate_up(g, u).to(DEV), out=out[:, : N // 2])
    xd = x.double()
    assert rel(out[:, : N // 2], O.silu(xd @ g.double().T) * (xd @ u.double().T)) < 3e-6 and out[:, N // 2 :].abs().sum() == 0


# ----------------------------------------------------------------------------- recurrence
def rglru_case(W, nb, taps, dtype, seed=0):
    """Padded weights (as the model lays them out) and the plain ones."""
    k, bs = W // nb, up(W // nb, 32)
    w = {"ra": rnd(nb, k, k, seed=1, std=2 * k ** -0.5, dtype=dtype), "ri": rnd(nb, k, k, seed=2, std=2 * k ** -0.5, dtype=dtype),
         "ra.b": rnd(nb, k, seed=3), "ri.b": rnd(nb, k, seed=4), "conv": rnd(W, taps, seed=5, std=0.6), "conv.b": rnd(W, seed=6, std=0.3),
         "x.b": rnd(W, seed=7, std=0.3), "y.b": rnd(W, seed=8, std=0.3), "lam": rnd(W, seed=9, std=2.5) - 4.0}

    def chan(t):
        o = torch.zeros(*t.shape[:-1], nb, bs)
        o[..., :k] = t.reshape(*t.shape[:-1], nb, k)
        return o.view(*t.shape[:-1], nb * bs)

    gates = torch.zeros(nb, 2, bs, bs, dtype=dtype)
    gates[:, 0, :k, :k], gates[:, 1, :k, :k] = w["ra"], w["ri"]
    dev = lambda t: chan(t).contiguous().to(DEV)  # noqa: E731
    p = mixers.RgLruWeights(nb=nb, yb=dev(w["y.b"]), xb=dev(w["x.b"]), conv=dev(w["conv"].t().contiguous()), conv_b=dev(w["conv.b"]),
                            gates=ops.gate_fragments(gates.to(DEV)), rb=dev(w["ra.b"].reshape(-1)), ib=dev(w["ri.b"].reshape(-1)),
                            decay=dev(-8.0 * torch.nn.functional.softplus(w["lam"])))
    return w, p, chan


RGLRU = [(60, 3, 4), (40, 1, 1), (256, 2, 3), (96, 3, 2), (512, 2, 4), (640, 2, 6), (33, 33, 3), (768, 1, 4)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,nb,taps", RGLRU)
@pytest.mark.parametrize("lens", [((2, 0, 1), (0, 5, 33), (3, 0, 64), (1, 100, 2), (4, 1, 95)), ((1, 0, 300), (0, 7, 257), (4, 2, 1)),
                                  ((3, 9, 1), (1, 0, 1), (0, 1, 1), (4, 40, 1)), ((2, 0, 2), (1, 3, 30), (0, 0, 17))], ids=["mix", "long", "one", "short"])
def test_rglru(dtype, W, nb, taps, lens):
    """Rows form (where the rows fit) and scan form over several runs: fresh ones, continuing ones (also with
    fewer tokens behind them than the convolution has taps), slow and fast channels."""
    w, p, chan = rglru_case(W, nb, taps, dtype)
    Wp = p.decay.numel()
    tot = sum(n for _, _, n in lens)
    y, x = rnd(tot, W, seed=11, dtype=dtype), rnd(tot, W, seed=12, dtype=dtype)
    st0 = rnd(5, taps, W, seed=13, std=2.0)
    want, end = torch.zeros(tot, W, dtype=torch.float64), st0.double().clone()
    wd = {k: v.double() for k, v in w.items()}
    r0 = 0
    ids, pos, runs = [], [], []
    for sid, p0, n in lens:
        xs = x[r0 : r0 + n].double() + wd["x.b"]
        before = st0[sid, 1:].double() if p0 else torch.zeros(taps - 1, W, dtype=torch.float64)
        u = O.causal_conv(xs, wd["conv"], wd["conv.b"], before).to(dtype).double()
        r = O.sigmoid(O.block_linear(u, wd["ra"]) + wd["ra.b"].reshape(-1))
        i = O.sigmoid(O.block_linear(u, wd["ri"]) + wd["ri.b"].reshape(-1))
        S = O.gated_linear_recurrence(u, r, i, wd["lam"], st0[sid, 0].double() if p0 else None)
        want[r0 : r0 + n] = S * O.gelu_tanh(y[r0 : r0 + n].double() + wd["y.b"])
        end[sid, 0], end[sid, 1:] = S[-1], torch.cat([before, xs])[n:]
        ids += [sid] * n
        pos += list(range(p0, p0 + n))
        runs.append((r0, n))
        r0 += n
    yx = torch.cat([chan(y.float()), chan(x.float())], 1).to(dtype).to(DEV)
    ids, pos = torch.tensor(ids, dtype=torch.int32, device=DEV), torch.tensor(pos, dtype=torch.int32, device=DEV)
    real = chan(torch.ones(W)).bool()
    for plan in ([None] if tot <= 64 else []) + [ops.plan_runs(runs, DEV, 400, scan_rows=mixers.SCAN_ROWS)]:
        st = chan(st0).reshape(5, -1).contiguous().to(DEV)
        out = torch.zeros(tot, Wp + 8, dtype=dtype, device=DEV)
        ops.rglru(yx, p, seq_ids=ids, positions=pos, slots=pos.long(), state=st, out=out[:, :Wp], plan=plan)
        # (bf16: u is rounded where the kernel rounds it; a near-tie of that rounding moves u by a unit)
        tol = 2e-5 if dtype == F32 else 1.2e-2
        assert rel(out[:, :Wp].cpu()[:, real], want) < tol
        assert rel(st.cpu().view(5, taps, Wp)[..., real], end) < tol
        assert out[:, Wp:].abs().sum() == 0 and out[:, :Wp].cpu()[:, ~real].abs().sum() == 0


@pytest.mark.parametrize("dtype", DTYPES)
def test_rglru_inert_rows(dtype):
    w, p, chan = rglru_case(256, 2, 3, dtype)
    yx = rnd(6, 512, seed=1, dtype=dtype).to(DEV)
    ids, pos = torch.tensor([1, 1, 0, 2, 0, 0], dtype=torch.int32, device=DEV), torch.tensor([4, 5, 0, 3, 0, 0], dtype=torch.int32, device=DEV)
    slots = torch.tensor([1, 1, -1, 1, -1, -1], device=DEV)
    st = rnd(3, 768, seed=2).to(DEV)
    st0 = st.clone()
    out = torch.full((6, 256), float("nan"), dtype=dtype, device=DEV)
    ops.rglru(yx, p, seq_ids=ids, positions=pos, slots=slots, state=st, out=out)
    live = [0, 1, 3]
    alone = torch.zeros(3, 256, dtype=dtype, device=DEV)
    st1 = st0.clone()
    ops.rglru(yx[live], p, seq_ids=ids[live], positions=pos[live], slots=slots[live], state=st1, out=alone)
    assert torch.equal(out[live], alone) and torch.equal(st, st1) and torch.equal(st[0], st0[0]) and not torch.equal(st[1], st0[1])
    assert out[[2, 4, 5]].abs().sum() == 0


# ----------------------------------------------------------------------------- latent attention
LATENT = [  # H, dim, rot, vd, rank, block size, n
    (3, 20, 6, 24, 40, 16, 150),
    (16, 64, 32, 64, 128, 16, 300),
    (1, 32, 10, 16, 33, 16, 90),
    (20, 40, 16, 40, 96, 32, 130),       # more heads than MFMA columns
    (8, 128, 64, 128, 512, 16, 200),
    (4, 96, 64, 80, 200, 16, 140),
    (6, 33, 66, 17, 64, 16, 70),         # a rotated part larger than the other
    (2, 32, 32, 32, 300, 16, 100),
    (3, 40, 16, 24, 700, 16, 90),
]


def latent_case(case, dtype, seed=0, own=True):
    H, dim, rot, vd, rank, bs, n = case
    D = dict(dim=up(dim, 32), rot=up(rot, 32), vd=up(vd, 16), rank=up(rank, 32))
    w = {"uk": rnd(H * dim, rank, seed=1, std=rank ** -0.5, dtype=dtype), "uv": rnd(H * vd, rank, seed=2, std=rank ** -0.5, dtype=dtype),
         "norm": 1 + rnd(rank, seed=3, std=0.2), "sink": rnd(H, seed=4) + 2.0}
    uk, uv = torch.zeros(H, D["rank"], D["dim"], dtype=dtype), torch.zeros(H, D["vd"], D["rank"], dtype=dtype)
    uk[:, :rank, :dim] = w["uk"].view(H, dim, rank).transpose(1, 2)
    uv[:, :vd, :rank] = w["uv"].view(H, vd, rank)
    p = mixers.LatentWeights(H=H, dim_p=D["dim"], rot_p=D["rot"], rank_p=D["rank"], vd=D["vd"], scale=0.25, eps=1e-3,
                             norm=w["norm"].to(DEV), sink=w["sink"].to(DEV), uk=ops.fragments(uk.to(DEV)), uv=ops.fragments(uv.to(DEV)))
    return w, p, D


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", LATENT, ids=str)
@pytest.mark.parametrize("M", [1, 37, 70])
def test_latent_qkv(dtype, case, M):
    H, dim, rot, vd, rank, bs, _ = case
    w, p, D = latent_case(case, dtype)
    hq, dk = D["dim"] + D["rot"], D["rank"] + D["rot"]
    q, c, kr = rnd(M, H, dim + rot, seed=5, dtype=dtype), rnd(M, rank, seed=6, std=3.0, dtype=dtype), rnd(M, rot, seed=7, dtype=dtype)
    y = torch.zeros(M, H * hq + dk + 16, dtype=dtype)
    yq = y[:, : H * hq].view(M, H, hq)
    yq[..., :dim], yq[..., D["dim"] : D["dim"] + rot] = q[..., :dim], q[..., dim:]
    y[:, H * hq : H * hq + rank], y[:, H * hq + D["rank"] : H * hq + D["rank"] + rot] = c, kr
    nb = 6
    pos = torch.arange(M, dtype=torch.int32) + 900
    slots = torch.randperm(nb * bs, generator=torch.Generator().manual_seed(0))[:M]
    if M > 5:
        slots[5] = -1
    cache = torch.zeros(nb, 1, bs, dk, dtype=dtype, device=DEV)
    out = torch.full((M, H * dk), float("nan"), dtype=dtype, device=DEV)
    rope = ops.rope_table(1000, rot, 250.0, device=DEV)
    args = dict(rope=rope, positions=pos.to(DEV), slots=slots.to(DEV))
    ops.latent_qkv(y.to(DEV), p, q_out=out, cache=cache, **args)
    tol = 3e-6 if dtype == F32 else 8e-3
    got = out.cpu().view(M, H, dk)
    lat = torch.einsum("mhi,hir->mhr", q[..., :dim].double(), w["uk"].double().view(H, dim, rank))
    assert rel(got[..., :rank], lat) < tol
    assert rel(got[..., D["rank"] : D["rank"] + rot], O.rotate(q[..., dim:].double(), 250.0, first=900)) < tol
    assert got[..., rank : D["rank"]].abs().sum() == 0 and got[..., D["rank"] + rot :].abs().sum() == 0
    rows = cache.cpu().view(nb * bs, dk)
    live = slots >= 0
    cw = O.rms_norm(c.double(), w["norm"].double(), 1e-3)
    kw = O.rotate(kr[:, None].double(), 250.0, first=900)[:, 0]
    assert rel(rows[slots[live], :rank], cw[live]) < tol and rel(rows[slots[live], D["rank"] : D["rank"] + rot], kw[live]) < tol
    assert int((rows != 0).any(-1).sum()) == int(live.sum())  # the inert row wrote nothing
    # a layer that reads another layer's cache: the same queries, no write
    again = torch.zeros_like(out)
    before = cache.clone()
    ops.latent_qkv(y.to(DEV), p, q_out=again, cache=None, **args)
    assert torch.equal(again, out) and torch.equal(cache, before)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M", [1, 16, 19, 70, 200])
@pytest.mark.parametrize("nb,N,K", [(3, 48, 32), (5, 272, 96), (2, 128, 512)])
def test_head_linear(dtype, M, nb, N, K):
    x, w = rnd(M, nb * (K + 32), seed=1, dtype=dtype), rnd(nb, N, K, seed=2, std=K ** -0.5, dtype=dtype)
    out = torch.zeros(M, nb * (N + 16), dtype=dtype, device=DEV)
    ops.ext().head_linear(x.to(DEV), K + 32, ops.fragments(w.to(DEV)), nb, N, K, out, N + 16)
    want = torch.einsum("mbk,bnk->mbn", x.view(M, nb, -1)[..., :K].double(), w.double())
    got = out.cpu().view(M, nb, -1)
    assert rel(got[..., :N], want) < (3e-6 if dtype == F32 else 8e-3) and got[..., N:].abs().sum() == 0


def attention_case(case, dtype):
    """One sequence's cached latents in scattered blocks (other blocks hold rubbish), queries in head space, some
    keys far above the others: at block and round borders, far back, and the first."""
    H, dim, rot, vd, rank, bs, n = case
    w, p, D = latent_case(case, dtype)
    dk = D["rank"] + D["rot"]
    gen = torch.Generator().manual_seed(3)
    c, kr = rnd(n, rank, seed=5), rnd(n, rot, seed=6, std=0.3)
    q = rnd(n, H, dim + rot, seed=7, std=0.3)
    q[..., dim] += 4.0
    for j in {0, 1, 15, 16, 31, 32, 63, 64, 65, n // 2, n - 20}:
        kr[j, 0] += 6.0 + 2 * float(torch.rand(1, generator=gen))
    c, kr, q = c.to(dtype), kr.to(dtype), q.to(dtype)
    nblk = -(-n // bs)
    perm = torch.randperm(nblk + 3, generator=gen)[:nblk].tolist()
    cache = rnd(nblk + 3, 1, bs, dk, seed=77, std=30.0, dtype=dtype)
    for j in range(n):
        row = torch.zeros(dk, dtype=dtype)
        row[:rank], row[D["rank"] : D["rank"] + rot] = c[j], kr[j]
        cache[perm[j // bs], 0, j % bs] = row
    table = torch.zeros(4, nblk + 2, dtype=torch.int32)
    table[2, :nblk] = torch.tensor(perm)
    gate = rnd(n, H * D["vd"], seed=8, dtype=dtype)
    k = (c.double() @ w["uk"].double().T).view(n, H, dim)
    v = (c.double() @ w["uv"].double().T).view(n, H, vd)
    causal = torch.ones(n, n).tril().bool()
    heads = []
    for h in range(H):
        s = (q[:, h, :dim].double() @ k[:, h].T + q[:, h, dim:].double() @ kr.double().T) * 0.25
        o = O.sink_softmax(s.masked_fill(~causal, float("-inf")), w["sink"][h].double()) @ v[:, h]
        heads.append(o * O.sigmoid(gate[:, h * D["vd"] : h * D["vd"] + vd].double()))
    return w, p, D, q, cache.to(DEV), table.to(DEV), gate.to(DEV), torch.stack(heads, 1)


def latent_queries(q, w, case, D, dtype):
    """The queries as latent_qkv leaves them: product with the key projection, rotated part behind it."""
    H, dim, rot, vd, rank, bs, n = case
    o = torch.zeros(n, H, D["rank"] + D["rot"])
    o[..., :rank] = torch.einsum("mhi,hir->mhr", q[..., :dim].float(), w["uk"].float().view(H, dim, rank))
    o[..., D["rank"] : D["rank"] + rot] = q[..., dim:].float()
    return o.view(n, -1).to(dtype).to(DEV)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", LATENT, ids=str)
def test_latent_attention(dtype, case):
    H, dim, rot, vd, rank, bs, n = case
    w, p, D, q, cache, table, gate, want = attention_case(case, dtype)
    qd = latent_queries(q, w, case, D, dtype)
    max_ctx = (table.shape[1] - 2) * bs
    sc = mixers.LatentScratch([(H, D["rank"])], max_ctx, DEV)
    pos = torch.arange(n, dtype=torch.int32, device=DEV)
    sid = torch.full((n,), 2, dtype=torch.int32, device=DEV)
    slots = torch.zeros(n, dtype=torch.int64, device=DEV)
    tol = 1e-5 if dtype == F32 else 2e-2

    def run(sel):
        sel = torch.tensor(sel, device=DEV)
        out = torch.full((len(sel), H * D["vd"]), float("nan"), dtype=dtype, device=DEV)
        ops.latent_attention(qd[sel], p, cache=cache, block_table=table, positions=pos[sel], seq_ids=sid[sel], slots=slots[sel],
                             gate=gate[sel], max_ctx=max_ctx, scratch=sc, out=out)
        return out.cpu().view(len(sel), H, D["vd"])

    for sel in (list(range(n)), [n - 1], [0], [0, 1, n - 1], [63, 64, 65, 16, 15, n // 2, n // 2 + 1]):
        got = run(sel)
        assert rel(got[..., :vd], want[sel]) < tol and got[..., vd:].abs().sum() == 0, sel
    # inert rows of a padded step are zero and touch nothing
    slots[5] = -1
    got = run(list(range(12)))
    assert got[5].abs().sum() == 0 and rel(got[:5, :, :vd], want[:5]) < tol


@pytest.mark.parametrize("case", LATENT, ids=str)
@pytest.mark.parametrize("cuts", [[(0, 1000)], [(7, 2), (30, 60), (3, 1), (-1, 1), (16, 49)], [(0, 33), (64, 64), (33, 31)], [(1, 40)]], ids=str)
def test_latent_prefill(case, cuts, monkeypatch):
    """The prefill form (context expanded to keys and values) of whole prompts, runs from the middle, short runs
    and single rows beside them."""
    H, dim, rot, vd, rank, bs, n = case
    w, p, D, q, cache, table, gate, want = attention_case(case, BF16)
    vdk = up(D["vd"], 32)
    kv = torch.zeros(H * (D["dim"] + vdk), up(D["rank"], 128), dtype=BF16)
    kv[: H * D["dim"]].view(H, D["dim"], -1)[:, :dim, :rank] = w["uk"].view(H, dim, rank)
    kv[H * D["dim"] :].view(H, vdk, -1)[:, :vd, :rank] = w["uv"].view(H, vd, rank)
    p.w_kv = ops.TiledWeight(kv.to(DEV))
    assert ops.ext().latent_prefill_fits(D["dim"], D["rot"], vdk)
    qd = latent_queries(q, w, case, D, BF16)
    y = torch.zeros(n, H, D["dim"] + D["rot"], dtype=BF16)
    y[..., :dim] = q[..., :dim]
    y = y.view(n, -1).to(DEV)
    max_ctx = (table.shape[1] - 2) * bs
    sc = mixers.LatentScratch([(H, D["rank"])], max_ctx, DEV)
    sel, runs = [], []
    for a, c in cuts:
        a = a % n
        c = min(c, n - a)
        runs.append((len(sel), c, 2, a))
        sel += list(range(a, a + c))
    monkeypatch.setattr(mixers, "EXPAND_ROWS", 16)
    plan = mixers.plan_latent(runs, DEV, ops.plan_runs(runs, DEV, n - 1))
    assert plan.q_tiles is not None and (plan.short is not None) == any(c < 16 for _, c, _, _ in runs)
    st = torch.tensor(sel, device=DEV)
    out = torch.full((len(sel), H * D["vd"]), float("nan"), dtype=BF16, device=DEV)
    ops.latent_attention(qd[st], p, cache=cache, block_table=table, positions=st.int(), seq_ids=torch.full_like(st, 2).int(),
                         slots=torch.zeros_like(st), gate=gate[st], max_ctx=max_ctx, scratch=sc, out=out, y=y[st], plan=plan)
    got = out.cpu().view(len(sel), H, D["vd"])
    assert rel(got[..., :vd], want[sel]) < 2e-2 and got[..., vd:].abs().sum() == 0


# ----------------------------------------------------------------------------- routed experts
MOE = [(8, 2, 40, 72), (5, 1, 128, 130), (16, 4, 96, 256), (3, 3, 64, 100), (40, 6, 32, 64), (1, 1, 48, 48), (130, 2, 16, 140)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,ff,d", MOE)
@pytest.mark.parametrize("M", [1, 7, 16, 40, 64, 150, 700])
def test_moe(dtype, E, top, ff, d, M, monkeypatch):
    """Every row's experts, their scores on the input side, the tables' bounds; some rows inert.  Every tile size
    that could serve the rows."""
    K, F, N = up(d, 128), up(ff, 128), up(d, 16)
    h = rnd(M, d, seed=1, dtype=dtype)
    router = rnd(E, d, seed=2, std=2 * d ** -0.5, dtype=dtype)
    s = O.sigmoid(h.double() @ router.double().T)
    for t in range(M):  # no close calls: the chosen ones stand apart
        if top < E:
            v = s[t].sort(descending=True).values
            if v[top - 1] - v[top] < 2e-3:
                h[t] = h[t - 1] if t else h[t]
    wg, wu, wd = rnd(E, ff, d, seed=3, std=d ** -0.5, dtype=dtype), rnd(E, ff, d, seed=4, std=d ** -0.5, dtype=dtype), rnd(E, d, ff, seed=5, std=ff ** -0.5, dtype=dtype)
    idx, val = O.route(h.double(), router.double(), top)
    want = torch.stack([torch.stack([O.expert(val[t, k] * h[t].double(), {"gate": wg[idx[t, k]].double(), "up": wu[idx[t, k]].double(),
                                                                          "down": wd[idx[t, k]].double()}) for k in range(top)]) for t in range(M)])
    gu = torch.zeros(E, 2 * F, K, dtype=dtype)
    for e in range(E):
        g, u = torch.zeros(F, K, dtype=dtype), torch.zeros(F, K, dtype=dtype)
        g[:ff, :d], u[:ff, :d] = wg[e], wu[e]
        gu[e] = ops.interleave_gate_up(g, u)
    dn = torch.zeros(E, N, F, dtype=dtype)
    dn[:, :d, :ff] = wd
    r = torch.zeros(up(E, 16), K, dtype=dtype)
    r[:E, :d] = router
    p = mixers.MoeWeights(E=E, top=top, router=ops.fragments(r.to(DEV)), gate_up=ops.tile_weights(gu.to(DEV)), down=ops.tile_weights(dn.to(DEV)))
    hp = torch.zeros(M, K, dtype=dtype)
    hp[:, :d] = h
    slots = torch.zeros(M, dtype=torch.int64, device=DEV)
    inert = [t for t in (2, M - 1) if M > 4]
    slots[inert] = -1
    for tile in [t for t in mixers.MOE_TILES if t <= 32 or (dtype == BF16 and M >= 40)]:
        monkeypatch.setattr(mixers, "moe_tile", lambda *_: tile)  # noqa: B023
        bufs = ops.moe_buffers(M, [(E, top, F)], dtype, DEV)
        for _ in range(2):  # (the tables are used again)
            out = torch.full((M * top, N), 7.0, dtype=dtype, device=DEV)
            ops.moe(hp.to(DEV), p, slots=slots, bufs=bufs, out=out)
            got = out.cpu().view(M, top, N)
            live = [t for t in range(M) if t not in inert]
            # (equal scores may come in either order: compare the sum, and each where the order is certain)
            assert rel(got[live][..., :d].double().sum(1), want[live].sum(1)) < (1e-5 if dtype == F32 else 2e-2)
            assert (got[inert] == 7.0).all()           # inert rows choose nothing
            assert int(bufs.ticket) == 0


# ----------------------------------------------------------------------------- the model through the engine
CFGS = {
    "odd": O.model_config(76, 101, [
        O.latent_layer(3, 20, 6, 24, 40, O.moe(5, 2, 24)),
        O.rglru_layer(60, 3, 4, O.dense(56)),
        O.latent_layer(5, 12, 6, 8, 40, None, scale=0.3, kv_from=0),
        O.rglru_layer(40, 1, 1, O.moe(4, 1, 40)),
        O.latent_layer(1, 32, 10, 16, 33, O.dense(33), base=500.0),
        O.latent_layer(2, 16, 6, 16, 40, O.moe(3, 3, 16), kv_from=0)], eps=1e-3),
    "even": O.model_config(384, 512, [
        O.rglru_layer(512, 4, 4, O.dense(512)),
        O.latent_layer(8, 64, 32, 64, 128, O.moe(8, 2, 128)),
        O.rglru_layer(256, 1, 3, O.moe(16, 4, 64)),
        O.latent_layer(12, 48, 32, 32, 128, O.dense(384), kv_from=1, scale=0.2)], scale=1.5),
    "one": O.model_config(130, 77, [O.rglru_layer(32, 32, 2, O.moe(1, 1, 9)), O.latent_layer(1, 1, 2, 11, 7, None)], scale=1.0),
    "recurrent": O.model_config(64, 50, [O.rglru_layer(48, 2, 3, O.dense(32)), O.rglru_layer(32, 1, 2, None)]),
}


def close(got, want, dtype):
    """Rounding apart, the same logits.  (bf16, narrow layers: a norm magnifies the rounding of a small branch now and
    then, so a few rows may be further off.)"""
    e = O.logit_error(got, want)
    if dtype == F32:
        return bool(e.max() < 3e-5)
    return bool(e.max() < 0.15 and (e > 0.04).double().mean() <= max(0.03, 1 / len(e)))


def tokens(n, seed, vocab):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


_MODELS = {}


def setup(name, dtype, **kw):
    if (name, dtype) not in _MODELS:
        w = O.random_weights(CFGS[name], 5)
        _MODELS[name, dtype] = (w, RipupelModel(RipupelConfig.from_json(CFGS[name]), weights=w, device=DEV, dtype=dtype))
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
        assert rel(g, r) < (1e-5 if dtype == F32 else 3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CFGS))
@pytest.mark.parametrize("cuts", [[300], [2], [16, 1], [70, 3, 2], [1], [200, 100], [130, 2]], ids=str)
def test_prompts_in_portions(name, dtype, cuts):
    n = 300 if max(cuts) > 100 else 150
    cfg, w, eng = setup(name, dtype)
    t, want = oracle(name, 300, 1)
    t, want = t[:n], want[:n]
    seq, out, i, k = eng.new_sequence([]), [], 0, 0
    while i < len(t):
        part = t[i : i + cuts[k % len(cuts)]]
        out.append(eng.step_batch([(seq, part)], range(len(part))).clone())
        i, k = i + len(part), k + 1
    assert close(torch.cat(out), want, dtype)


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
            k = int(rng.choice([1, 2, 30, 64, 150] if big else [1, 1, 2, 5, 17]))
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
        assert close(torch.cat(got[n]), reqs[n][1], dtype), n


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    """Decoding through the captured step graph, its first replay included (the capture's warm-up forwards must
    not advance the recurrent state)."""
    t, want = oracle("even", 260, 4)
    cfg, w, eng = setup("even", dtype)
    seq = eng.new_sequence([])
    out = [eng.step_batch([(seq, t[:5])], range(5)).clone()]
    for i in range(5, 260):
        out.append(eng.step_batch([(seq, t[i : i + 1])], [0]).clone())
    assert eng.stats["graph_replays"] >= 250
    assert close(torch.cat(out), want, dtype)


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


@pytest.mark.parametrize("cut", [0, 70, 199])
def test_far_keys_in_prompts_and_decoding(cut):
    """One attention layer (the recurrence's output taken out) whose query of the last token points at one far
    key: the logits change with that token, wherever it lies, and with the first token."""
    cfg = O.model_config(128, 64, [O.latent_layer(4, 32, 16, 32, 64, O.dense(64))])
    w = O.random_weights(cfg, 8)
    m = RipupelModel(RipupelConfig.from_json(cfg), weights=w, device=DEV, dtype=F32)
    eng = LLMEngine(m, max_seqs=2, max_model_len=256)
    t = tokens(201, 3, 64)

    def last(tt):
        s = eng.new_sequence([], use_prefix_cache=False)
        if cut:
            eng.step_batch([(s, tt[:cut])])
            for x in tt[cut:-1]:
                eng.step_batch([(s, [x])])
            r = eng.step_batch([(s, tt[-1:])], [0]).clone()
        else:
            r = eng.step_batch([(s, tt)], [len(tt) - 1]).clone()
        eng.free_sequence(s, publish=False)
        return r

    base = last(t)
    for j in (0, 1, 15, 16, 63, 64, 127, 128, 199):
        tt = list(t)
        tt[j] = (tt[j] + 1) % 64
        d = last(tt) - base
        want = O.forward(cfg, w, tt)[-1:] - O.forward(cfg, w, t)[-1:]
        assert float(d.abs().max()) > 1e-4 and rel(d, want) < 2e-2, j


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_scheduler(dtype):
    cfg, w, eng = setup("even", dtype, max_seqs=2)
    prompts = [tokens(n, 40 + n, 512) for n in (37, 3, 90)]
    outs = TokenScheduler(eng, token_budget=80).generate(prompts, 8)
    for p, o in zip(prompts, outs):
        want = O.forward(cfg, w, p + o)
        for i, tok in enumerate(o):  # (each token is the oracle's choice given the tokens before it, up to near-ties)
            row = want[len(p) - 1 + i]
            assert row.max() - row[tok] < (1e-4 if dtype == F32 else 0.1) * row.std(), (i, tok)


def test_sampling_at_a_temperature_is_reproducible():
    _, _, eng = setup("even", BF16, max_seqs=2)
    p = tokens(20, 1, 512)
    a, b = (TokenScheduler(eng, temperature=300.0, seed=s).generate([p], 12)[0] for s in (3, 3))
    c = TokenScheduler(eng, temperature=300.0, seed=4).generate([p], 12)[0]
    assert a == b and a != c


def test_trace_replay_command(tmp_path):
    cfg = CFGS["odd"]
    w = O.random_weights(cfg, 5)
    O.save_model(str(tmp_path / "m"), cfg, w)
    t, want = oracle("odd", 150, 1)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": t[:100], "want": [99, 7]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": t[100:], "want": [49]}, {"id": "b", "tokens": t[:2], "want": [1]}],
              "end": ["a", "b"]}]
    for dtype, dt in (("bfloat16", BF16), ("float32", F32)):
        r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype, "--out",
                            str(tmp_path / dtype), "--max-tokens", "256"], input="".join(json.dumps(s) + "\n" for s in steps),
                           capture_output=True, text=True, timeout=100)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [x for x in r.stdout.split("\n") if x.startswith("done")] == ["done 0", "done 1"]
        got = torch.cat([torch.from_numpy(np.fromfile(tmp_path / dtype / f"{i}.f32", dtype="<f4")).view(-1, 101) for i in (0, 1)])
        assert close(got, want[[99, 7, 149, 1]], dt)


def test_generate_command(tmp_path):
    cfg = CFGS["odd"]
    O.save_model(str(tmp_path / "m"), cfg, O.random_weights(cfg, 5))
    r = subprocess.run([sys.executable, "-m", "voice_enabled_browser_automation_amd.generate", "--model", str(tmp_path / "m"), "--ids",
                        "5,6,7", "--ids", "9", "--max-new", "4", "--max-model-len", "64"], capture_output=True, text=True,
                       timeout=100, cwd=ROOT)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [len(json.loads(x)["tokens"]) for x in r.stdout.split("\n") if x.startswith("{")] == [4, 4]


def test_intent_engine_serves_a_ripupel_preset():
    from voice_enabled_browser_automation_amd.brain.intent_engine import LLMIntentEngine
    from voice_enabled_browser_automation_amd.contracts import ParseResponse, safe_parse
    from voice_enabled_browser_automation_amd.runtime.weights import load_llm
    from voice_enabled_browser_automation_amd.tokenizer import load_tokenizer

    eng = LLMEngine(load_llm("ripupel-tiny", device=DEV), max_seqs=4, max_model_len=2048)
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
