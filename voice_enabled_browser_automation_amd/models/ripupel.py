"""Ripupel decoder: serial layers of a real-gated linear recurrence or latent attention, each followed by
a dense feed-forward or routed experts, with a norm before and after every sublayer.

    x <- x + norm1b(mixer(norm1(x)));  x <- x + norm2b(ff(norm2(x)))        (layer norms, weight only)

Engine contract as models/kabanex.py: ragged rows with their own position, slot and block-table row,
paged cache rows per attention layer ([latent | rotated key part]; a layer may read an earlier layer's),
one f32 state row per sequence and recurrent layer ([S | the convolution's last inputs]).

Launches of a decode step (T activations, f32 residual, branch outputs T):

    recurrent mixer   input projection [y | x] -> convolution + gates + recurrence -> output projection
    latent attention  input projection [q | latent | key part | gate] -> queries into latent space, rotation,
                      latent norm, cache write -> attention over the cached latents -> merge with the sinks,
                      value projection, gate -> output projection
                      (prompt-sized runs instead expand their context's keys and values once: gather -> GEMM ->
                      flash attention with sinks and gate)
    dense ff          gate / up with SwiGLU in the epilogue -> down
    routed experts    router + grouping -> gate / up of the chosen experts -> down, a row per (token, expert)

and one launch between two sublayers: the branch's norm, the residual sum (over the experts' rows) and the
next sublayer's norm.

Sizes are arbitrary: blocks of recurrence channels, head sizes and the latent are padded to 32, values to
16, projection inputs to 128, with zero weight rows / columns, so the padding contributes zeros.
"""
from __future__ import annotations

from dataclasses import dataclass
from types import SimpleNamespace
from typing import Dict, List, Optional, Sequence, Tuple

import torch

from .. import ops
from ..ops.mixers import SCAN_ROWS, LatentScratch, LatentWeights, MoeWeights, RgLruWeights, plan_latent
from ..parallel.tp import TPContext
from ..runtime.kv_cache import CacheLayer
from .config import DenseFFConfig, LatentAttentionConfig, MoEConfig, RgLruConfig, RipupelConfig


def _up(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def _columns(n: int) -> int:
    """Rows of a fused projection weight: large ones fill the tiled GEMM's 256-column tile."""
    return _up(n, 256) if n >= 2048 else n


@dataclass(frozen=True)
class RgLruDims:
    nb: int
    block: int
    bs: int       # block, padded to 32

    @property
    def w(self) -> int:
        return self.nb * self.bs

    @property
    def n_in(self) -> int:
        return _columns(2 * self.w)

    @property
    def cols(self) -> int:
        return self.w


@dataclass(frozen=True)
class LatentDims:
    H: int
    dim: int      # unrotated part of a head, padded to 32
    rot: int      # rotated part, padded to 32
    vd: int       # values of a head, padded to 16
    rank: int     # latent, padded to 32
    own: bool     # has a latent of its own

    @property
    def at(self) -> Tuple[int, int]:
        """Columns of the latent and of the gate in the input projection (q is at 0)."""
        c = self.H * (self.dim + self.rot)
        return c, c + (self.rank + self.rot if self.own else 0)

    @property
    def n_in(self) -> int:
        return _columns(_up(self.at[1] + self.H * self.vd, 16))

    @property
    def cols(self) -> int:
        return self.H * self.vd

    @property
    def dk(self) -> int:
        return self.rank + self.rot


def _dims(m):
    if isinstance(m, RgLruConfig):
        return RgLruDims(nb=m.blocks, block=m.block, bs=_up(m.block, 32))
    return LatentDims(H=m.heads, dim=_up(m.dim, 32), rot=_up(m.rot_dim, 32), vd=_up(m.vdim, 16), rank=_up(m.kv_rank, 32),
                      own=m.kv_from is None)


@dataclass
class RipupelLayerWeights:
    norm1: torch.Tensor
    norm1b: torch.Tensor
    norm2: Optional[torch.Tensor]
    norm2b: Optional[torch.Tensor]
    w_in: object                 # [n_in, d_pad]
    w_out: object                # [n_out, cols padded to 128]
    mixer: object                # RgLruWeights | LatentWeights
    gate_up: object = None       # dense: interleaved [2 F, d_pad]
    down: object = None          # dense: [n_out, F]
    moe: Optional[MoeWeights] = None


class RipupelModel:
    shared_buffers = ("latent",)  # step buffers that ragged forwards use as well

    def __init__(self, cfg: RipupelConfig, *, device="cpu", dtype: Optional[torch.dtype] = None,
                 tp: Optional[TPContext] = None, seed: int = 0, weights: Optional[dict] = None):
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype or (torch.bfloat16 if self.device.type == "cuda" else torch.float32)
        if self.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"unsupported dtype {self.dtype} (bfloat16 | float32)")
        self.tp = tp or TPContext.single()
        assert self.tp.size == 1, "Ripupel runs on one GPU"
        # a recurrent state cannot be resumed from prefix-cached blocks
        self.stateful = any(isinstance(L.mixer, RgLruConfig) for L in cfg.layers)
        self.dims = [_dims(L.mixer) for L in cfg.layers]
        self.ffs = [_up(L.mlp.ff, 128) if L.mlp is not None else 0 for L in cfg.layers]
        self.d_pad = _up(cfg.hidden, 128)
        self.n_out = _up(cfg.hidden, 16)
        self.v_pad = _up(cfg.vocab_size, 16)
        self.v_start, self.v_end = 0, cfg.vocab_size
        self.ropes: Dict[Tuple[float, int], torch.Tensor] = {}
        self._old_ropes: List[torch.Tensor] = []
        self.ensure_positions(cfg.max_pos)
        self._build(weights if weights is not None else _RandomWeights(cfg, seed, self.device))

    # ------------------------------------------------------------------ weights
    def _build(self, w) -> None:
        cfg, dev, dt, d = self.cfg, self.device, self.dtype, self.cfg.hidden
        gpu = dev.type == "cuda"
        tiled = gpu and dt == torch.bfloat16
        place = (lambda t: ops.TiledWeight(t)) if tiled else (lambda t: t)
        frag = ops.fragments if gpu else (lambda t: t)

        def get(name, shape, dtype):
            t = w[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"{name}: shape {tuple(t.shape)}, expected {tuple(shape)}")
            return t.to(device=dev, dtype=dtype)

        mat = lambda name, *shape: get(name, shape, dt)                              # noqa: E731
        vec = lambda name, *shape: get(name, shape, torch.float32).contiguous()      # noqa: E731
        zeros = lambda *shape: torch.zeros(*shape, dtype=dt, device=dev)             # noqa: E731

        self.embed = mat("embed", cfg.vocab_size, d).contiguous()
        self.layers: List[RipupelLayerWeights] = []
        for i, (L, D) in enumerate(zip(cfg.layers, self.dims)):
            p, m = f"l{i}.", f"l{i}.mix."
            w_in = zeros(D.n_in, self.d_pad)
            w_out = zeros(self.n_out, _up(D.cols, 128))
            if isinstance(D, RgLruDims):
                mixer = self._build_rglru(L.mixer, D, m, mat, vec, zeros, w_in, w_out, gpu)
            else:
                mixer = self._build_latent(L.mixer, D, m, mat, vec, zeros, w_in, w_out, frag, tiled)
            lw = RipupelLayerWeights(norm1=vec(p + "norm1", d), norm1b=vec(p + "norm1b", d), norm2=None, norm2b=None,
                                     w_in=place(w_in), w_out=place(w_out), mixer=mixer)
            if L.mlp is not None:
                lw.norm2, lw.norm2b = vec(p + "norm2", d), vec(p + "norm2b", d)
                F = self.ffs[i]

                def expert(q):
                    g, u, dn = zeros(F, self.d_pad), zeros(F, self.d_pad), zeros(self.n_out, F)
                    g[: L.mlp.ff, :d], u[: L.mlp.ff, :d] = mat(q + "gate", L.mlp.ff, d), mat(q + "up", L.mlp.ff, d)
                    dn[:d, : L.mlp.ff] = mat(q + "down", d, L.mlp.ff)
                    return ops.interleave_gate_up(g, u), dn

                if isinstance(L.mlp, DenseFFConfig):
                    gu, dn = expert(p + "mlp.")
                    lw.gate_up, lw.down = place(gu), place(dn)
                else:
                    E = L.mlp.experts
                    r = zeros(_up(E, 16), self.d_pad)
                    r[:E, :d] = mat(p + "mlp.router", E, d)
                    gu, dn = zeros(E, 2 * F, self.d_pad), zeros(E, self.n_out, F)
                    for e in range(E):
                        a, b = expert(p + f"mlp.e{e}.")
                        gu[e : e + 1] = ops.tile_weights(a[None]) if gpu else a
                        dn[e : e + 1] = ops.tile_weights(b[None]) if gpu else b
                    lw.moe = MoeWeights(E=E, top=L.mlp.top, router=frag(r), gate_up=gu, down=dn)
            self.layers.append(lw)
        self.final_w = vec("final.norm", d)
        head = zeros(self.v_pad, self.d_pad)
        head[: cfg.vocab_size, :d] = self.embed
        self.lm_head = place(head)

    def _build_rglru(self, c: RgLruConfig, D: RgLruDims, m: str, mat, vec, zeros, w_in, w_out, gpu: bool) -> RgLruWeights:
        d, W, nb, k, bs, dev = self.cfg.hidden, c.width, D.nb, D.block, D.bs, self.device
        for at, name in ((0, "y"), (D.w, "x")):
            w_in[at : at + D.w].view(nb, bs, -1)[:, :k, :d] = mat(m + name, W, d).view(nb, k, d)
        w_out[:d, : D.w].view(d, nb, bs)[:, :, :k] = mat(m + "o", d, W).view(d, nb, k)

        def chan(t):  # f32 [.., width] -> padded channels
            o = torch.zeros(*t.shape[:-1], nb, bs, dtype=torch.float32, device=dev)
            o[..., :k] = t.view(*t.shape[:-1], nb, k)
            return o.view(*t.shape[:-1], D.w).contiguous()

        gates = zeros(nb, 2, bs, bs)
        gates[:, 0, :k, :k], gates[:, 1, :k, :k] = mat(m + "ra", nb, k, k), mat(m + "ri", nb, k, k)
        lam = vec(m + "lam", W).double()
        decay = (-8.0 * torch.nn.functional.softplus(lam)).float()
        return RgLruWeights(nb=nb, yb=chan(vec(m + "y.b", W)), xb=chan(vec(m + "x.b", W)),
                            conv=chan(vec(m + "conv", W, c.conv).t().contiguous()), conv_b=chan(vec(m + "conv.b", W)),
                            gates=ops.gate_fragments(gates) if gpu else gates, rb=chan(vec(m + "ra.b", nb, k).view(-1)),
                            ib=chan(vec(m + "ri.b", nb, k).view(-1)), decay=chan(decay))

    def _build_latent(self, c: LatentAttentionConfig, D: LatentDims, m: str, mat, vec, zeros, w_in, w_out, frag,
                      tiled: bool) -> LatentWeights:
        d, H, hq = self.cfg.hidden, c.heads, c.dim + c.rot_dim
        kv_at, g_at = D.at
        q = mat(m + "q", H * hq, d).view(H, hq, d)
        wq = w_in[: H * (D.dim + D.rot)].view(H, D.dim + D.rot, -1)
        wq[:, : c.dim, :d], wq[:, D.dim : D.dim + c.rot_dim, :d] = q[:, : c.dim], q[:, c.dim :]
        if D.own:
            dkv = mat(m + "dkv", c.kv_rank + c.rot_dim, d)
            w_in[kv_at : kv_at + c.kv_rank, :d] = dkv[: c.kv_rank]
            w_in[kv_at + D.rank : kv_at + D.rank + c.rot_dim, :d] = dkv[c.kv_rank :]
        w_in[g_at : g_at + H * D.vd].view(H, D.vd, -1)[:, : c.vdim, :d] = mat(m + "g", H * c.vdim, d).view(H, c.vdim, d)
        w_out[:d, : H * D.vd].view(d, H, D.vd)[:, :, : c.vdim] = mat(m + "o", d, H * c.vdim).view(d, H, c.vdim)
        uk, uv = zeros(H, D.rank, D.dim), zeros(H, D.vd, D.rank)
        uk[:, : c.kv_rank, : c.dim] = mat(m + "uk", H * c.dim, c.kv_rank).view(H, c.dim, c.kv_rank).transpose(1, 2)
        uv[:, : c.vdim, : c.kv_rank] = mat(m + "uv", H * c.vdim, c.kv_rank).view(H, c.vdim, c.kv_rank)
        w_kv = None
        if tiled:  # the same projections for prompts: keys of all heads, then values (32-column heads)
            vdk = _up(D.vd, 32)
            w_kv = zeros(_columns(H * (D.dim + vdk)), _up(D.rank, 128))
            w_kv[: H * D.dim, : D.rank].view(H, D.dim, D.rank).copy_(uk.transpose(1, 2))
            w_kv[H * D.dim : H * (D.dim + vdk), : D.rank].view(H, vdk, D.rank)[:, : D.vd] = uv
            w_kv = ops.TiledWeight(w_kv)
        return LatentWeights(H=H, dim_p=D.dim, rot_p=D.rot, rank_p=D.rank, vd=D.vd, scale=c.scale, eps=self.cfg.norm_eps,
                             norm=vec(m + "dkv.norm", c.kv_rank) if D.own else None, sink=vec(m + "sink", H), uk=frag(uk),
                             uv=frag(uv), w_kv=w_kv)

    def weight_bytes(self) -> int:
        ts = [self.lm_head]
        for L in self.layers:
            ts += [L.w_in, L.w_out]
            ts += [L.mixer.gates] if isinstance(L.mixer, RgLruWeights) else [L.mixer.uk, L.mixer.uv]
            ts += [t for t in (L.gate_up, L.down) if t is not None]
            ts += [L.moe.router, L.moe.gate_up, L.moe.down] if L.moe else []
        return sum(t.numel() * t.element_size() for t in ts)

    # ------------------------------------------------------------------ engine hooks
    def ensure_positions(self, n: int) -> None:
        """Rotation tables (one per distinct base and size) for at least n positions."""
        for L in self.cfg.layers:
            if not isinstance(L.mixer, LatentAttentionConfig):
                continue
            key = (L.mixer.rot_base, L.mixer.rot_dim)
            t = self.ropes.get(key)
            if t is None or t.shape[0] < n:
                if t is not None:
                    self._old_ropes.append(t)  # (another engine's captured graphs may hold its address)
                self.ropes[key] = ops.rope_table(n, key[1], key[0], device=self.device)

    def cache_layers(self) -> List[CacheLayer]:
        out = []
        for L, D in zip(self.cfg.layers, self.dims):
            if isinstance(D, RgLruDims):
                out.append(CacheLayer(state=L.mixer.conv * D.w))
            else:
                out.append(CacheLayer(n_kv_heads=1, k_dim=D.dk, v_dim=0, shared=L.mixer.kv_from))
        return out

    def row_buffers(self, rows: int, max_ctx: int) -> Dict[str, object]:
        """Activation buffers of a step of ``rows`` rows (fixed addresses when the engine keeps them)."""
        dev, dt = self.device, self.dtype
        e = lambda *n, t=dt: torch.empty(*n, dtype=t, device=dev)  # noqa: E731
        # every buffer is written before it is read, but for the padding columns of a mixer's output row: zeroed
        # once, never written (so each distinct layout has rows of its own)
        cols = {D.cols for D in self.dims}
        moes = [(L.mlp.experts, L.mlp.top, F) for L, F in zip(self.cfg.layers, self.ffs) if isinstance(L.mlp, MoEConfig)]
        parts = max([1] + [t for _, t, _ in moes])
        lat = [D.H * D.dk for D in self.dims if isinstance(D, LatentDims)]
        dense = [F for L, F in zip(self.cfg.layers, self.ffs) if isinstance(L.mlp, DenseFFConfig)]
        return dict(hidden=e(rows, self.d_pad, t=torch.float32), normed=e(rows, self.d_pad),
                    mix=e(rows * max(D.n_in for D in self.dims)), q=e(rows * max(lat)) if lat else None,
                    cat={c: e(rows, c) if c % 128 == 0 else torch.zeros(rows, _up(c, 128), dtype=dt, device=dev) for c in cols},
                    # (rows of pairs no token chose -- padded rows of a step graph -- are never written)
                    branch=torch.zeros(rows * parts, self.n_out, dtype=dt, device=dev),
                    act=e(rows * max(dense)) if dense else None,
                    moe=ops.moe_buffers(rows, moes, dt, dev) if moes else None)

    def step_buffers(self, rows: int, max_ctx: int) -> Dict[str, object]:
        dev = self.device
        b = self.row_buffers(rows, max_ctx)
        lat = [(D.H, D.rank) for D in self.dims if isinstance(D, LatentDims)]
        b.update(hidden_sel=torch.zeros(rows, self.d_pad, dtype=torch.float32, device=dev),
                 head_in=torch.zeros(rows, self.d_pad, dtype=self.dtype, device=dev),
                 logits_local=torch.zeros(rows, self.v_pad, dtype=torch.float32, device=dev),
                 latent=LatentScratch(lat, max_ctx, dev) if lat else None)
        return b

    def plan_rows(self, runs: Sequence[Tuple[int, int, int, int]], max_pos: int) -> SimpleNamespace:
        return plan_latent(runs, self.device, ops.plan_runs(runs, self.device, max_pos, scan_rows=SCAN_ROWS))

    # ------------------------------------------------------------------ forward
    def forward(self, bufs, M: int, kv, *, n_sel: Optional[int] = None, head: bool = True) -> torch.Tensor:
        """M ragged rows (bufs: tokens, positions, seq_ids, slots; ``plan`` for prompt-sized steps) ->
        f32 logits, or the residual rows with head=False (all, or those in bufs.sel[:n_sel])."""
        x, h = bufs.hidden[:M], bufs.normed[:M]
        plan = getattr(bufs, "plan", None)
        rows = dict(positions=bufs.positions[:M], seq_ids=bufs.seq_ids[:M], slots=bufs.slots[:M])
        ops.embedding_f32(bufs.tokens[:M], self.embed, out=x, scale=self.cfg.embed_scale)
        ops.layernorm_f32(x, self.layers[0].norm1, None, eps=self.cfg.norm_eps, out=h)
        for li in range(self.cfg.n_layers):
            self._layer(li, bufs, M, kv, x, h, rows, plan)
        if n_sel is not None:
            x = torch.index_select(x, 0, bufs.sel[:n_sel], out=bufs.hidden_sel[:n_sel])
        return self.lm_logits(bufs, x) if head else x

    def _layer(self, li: int, bufs, M: int, kv, x, h, rows, plan) -> None:
        """One layer of normed rows h (norm1 of x); leaves the next layer's in h."""
        C, D, L, eps = self.cfg.layers[li], self.dims[li], self.layers[li], self.cfg.norm_eps
        y = bufs.mix[: M * D.n_in].view(M, D.n_in)
        ops.linear(h, L.w_in, out=y)
        cat, br = bufs.cat[D.cols][:M], bufs.branch
        if isinstance(D, RgLruDims):
            ops.rglru(y, L.mixer, state=kv.state[li], out=cat[:, : D.cols], plan=plan, **rows)
        else:
            self._attend(li, y, cat[:, : D.cols], bufs, M, kv, rows, plan)
        ops.linear(cat, L.w_out, out=br[:M])
        after = self.layers[li + 1].norm1 if li + 1 < self.cfg.n_layers else None
        if C.mlp is None:
            ops.add_norm(x, br[:M], L.norm1b, after, eps=eps, out=h)
            return
        ops.add_norm(x, br[:M], L.norm1b, L.norm2, eps=eps, out=h)
        parts = 1
        if L.moe is not None:
            parts = L.moe.top
            ops.moe(h, L.moe, slots=rows["slots"], bufs=bufs.moe, out=br[: M * parts])
        else:
            act = bufs.act[: M * self.ffs[li]].view(M, self.ffs[li])
            ops.linear_swiglu(h, L.gate_up, out=act)
            ops.linear(act, L.down, out=br[:M])
        ops.add_norm(x, br[: M * parts], L.norm2b, after, eps=eps, out=h, n_parts=parts)

    def _attend(self, li: int, y, out, bufs, M: int, kv, rows, plan) -> None:
        a, D, w = self.cfg.layers[li].mixer, self.dims[li], self.layers[li].mixer
        g = D.at[1]
        q = ops.latent_qkv(y, w, rope=self.ropes[(a.rot_base, a.rot_dim)], positions=rows["positions"], slots=rows["slots"],
                           q_out=bufs.q[: M * D.H * D.dk].view(M, D.H * D.dk), cache=kv.k[li] if D.own else None, plan=plan)
        ops.latent_attention(q, w, cache=kv.k[li], block_table=bufs.block_table, gate=y[:, g : g + D.cols], max_ctx=bufs.max_ctx,
                             scratch=bufs.latent, out=out, y=y, plan=plan, **rows)

    def lm_logits(self, bufs, hs: torch.Tensor, col_mask: Optional[torch.Tensor] = None, mask_rows: int = 1,
                  gather: bool = True) -> torch.Tensor:
        """Final norm + the embedding table as LM head of residual rows -> f32 logits [rows, vocab] (contract as
        LlamaModel.lm_logits)."""
        n = hs.shape[0]
        fits = n <= bufs.logits_local.shape[0]
        h = bufs.head_in[:n] if fits else torch.empty(n, self.d_pad, dtype=self.dtype, device=hs.device)
        out = bufs.logits_local[:n] if fits else torch.empty(n, self.v_pad, dtype=torch.float32, device=hs.device)
        ops.layernorm_f32(hs, self.final_w, None, eps=self.cfg.norm_eps, out=h)
        if col_mask is not None and (self.dtype != torch.bfloat16 or col_mask.shape[1] * 32 < self.v_pad):
            col_mask = None
        ops.linear(h, self.lm_head, out=out, out_dtype=torch.float32, col_mask=col_mask, mask_rows=mask_rows)
        return out[:, : self.cfg.vocab_size]


class _RandomWeights:
    """Random tensors under the checkpoint's names, made on access (deterministic per name)."""

    def __init__(self, cfg: RipupelConfig, seed: int, device):
        self.cfg, self.seed, self.device = cfg, seed, device
        d, s = cfg.hidden, {}
        s["embed"], s["final.norm"] = (cfg.vocab_size, d), (d,)
        for i, L in enumerate(cfg.layers):
            p, m, c = f"l{i}.", f"l{i}.mix.", L.mixer
            s[p + "norm1"] = s[p + "norm1b"] = (d,)
            if isinstance(c, RgLruConfig):
                W, nb, k = c.width, c.blocks, c.block
                s.update({m + "y": (W, d), m + "y.b": (W,), m + "x": (W, d), m + "x.b": (W,), m + "conv": (W, c.conv),
                          m + "conv.b": (W,), m + "ra": (nb, k, k), m + "ra.b": (nb, k), m + "ri": (nb, k, k), m + "ri.b": (nb, k),
                          m + "lam": (W,), m + "o": (d, W)})
            else:
                H = c.heads
                s.update({m + "q": (H * (c.dim + c.rot_dim), d), m + "uk": (H * c.dim, c.kv_rank), m + "uv": (H * c.vdim, c.kv_rank),
                          m + "sink": (H,), m + "g": (H * c.vdim, d), m + "o": (d, H * c.vdim)})
                if c.kv_from is None:
                    s.update({m + "dkv": (c.kv_rank + c.rot_dim, d), m + "dkv.norm": (c.kv_rank,)})
            if L.mlp is None:
                continue
            s[p + "norm2"] = s[p + "norm2b"] = (d,)
            qs = [p + "mlp."]
            if isinstance(L.mlp, MoEConfig):
                s[p + "mlp.router"] = (L.mlp.experts, d)
                qs = [p + f"mlp.e{e}." for e in range(L.mlp.experts)]
            for q in qs:
                s.update({q + "gate": (L.mlp.ff, d), q + "up": (L.mlp.ff, d), q + "down": (d, L.mlp.ff)})
        self.shapes = s

    def __getitem__(self, name: str) -> torch.Tensor:
        shape = self.shapes[name]
        gen = torch.Generator(device=self.device)
        gen.manual_seed(self.seed * 1000003 + sum(ord(c) * 131 ** (i % 8) for i, c in enumerate(name)) % (1 << 31))
        t = torch.empty(shape, device=self.device, dtype=torch.float32).normal_(0.0, self.cfg.init_std, generator=gen)
        last = name.rsplit(".", 1)[-1]
        if last.startswith("norm"):
            t += 1.0
        elif last == "lam":      # decays of a trained recurrence: slow to fast channels
            t.uniform_(-7.0, 0.0, generator=gen)
        elif last == "conv":
            t[:, -1] += 1.0
        return t
