"""Kabanex decoder: parallel layers of windowed talking-heads attention, a minGRU and a squared-ReLU
feed-forward, all reading one LayerNorm of an f32 residual stream.

    h = LN(x);  x <- x + left_scale * attention(h) + right_scale * minGRU(h) + ff(h)

Engine contract as models/llama.py (ragged rows with their own position, slot and block-table row;
optional logit-row selection), plus a recurrent state row per sequence (``stateful``) next to the
paged K / V (``cache_layers``).  MI355X layout of a layer -- six launches at decode:

    layernorm_f32 -> ONE input projection [q | k | v | gate | z | x | g || up] whose epilogue squares the
    feed-forward part straight into the output projection's input -> rotation + cache write and the
    minGRU (right_scale in its epilogue, into that same input) -> attention (two launches: scores, then
    mixing and values; gate and left_scale in the epilogue, into that same input) -> ONE output projection over [heads | recurrence | feed-forward] with the f32 residual
    in its epilogue

Sizes are arbitrary: projection sections are padded to the MFMA tiles with zero weight rows / columns
(head sizes: q / k to 32, v to 16), so every kernel runs whole tiles and the padding contributes zeros.
"""
from __future__ import annotations

from dataclasses import dataclass
from types import SimpleNamespace
from typing import Dict, List, Optional, Sequence, Tuple

import torch

from .. import ops
from ..parallel.tp import TPContext
from ..runtime.kv_cache import CacheLayer
from .config import KabanexConfig, ParallelLayerConfig


def _up(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def _padded_heads(a) -> int:
    return (1 << (a.kv_heads - 1).bit_length()) * (1 << (a.heads // a.kv_heads - 1).bit_length())


@dataclass(frozen=True)
class LayerDims:
    """Padded section sizes of a layer's fused projections."""
    H: int
    G: int
    dk: int       # q / k head size, padded to 32
    dv: int       # v head size, padded to 16
    gate: int     # gate columns
    w: int        # recurrence channels, padded
    f: int        # feed-forward columns, padded (0: none)
    d: int        # input width, padded to 128

    @staticmethod
    def of(cfg: KabanexConfig, L: ParallelLayerConfig) -> "LayerDims":
        a = L.left
        return LayerDims(H=a.heads, G=a.kv_heads, dk=_up(a.dim, 32), dv=_up(a.vdim, 16), gate=_up(a.heads, 16),
                         w=_up(L.right.width, 16), f=_up(L.ffn, 16), d=_up(cfg.hidden, 128))

    @property
    def at(self) -> Tuple[int, int, int, int, int, int]:
        """Columns of k, v, gate, z, x, g in the input projection (q is at 0)."""
        k = self.H * self.dk
        v = k + self.G * self.dk
        gate = v + self.G * self.dv
        z = gate + self.gate
        return k, v, gate, z, z + self.w, z + 2 * self.w

    @property
    def n_mix(self) -> int:
        """Columns of the mixers' part; large projections are padded here to 256 columns in all (the tiled
        GEMM's large tile)."""
        n = self.at[5] + self.w
        return n if n + self.f < 2048 else _up(n + self.f, 256) - self.f

    @property
    def heads_out(self) -> int:
        return self.H * self.dv

    @property
    def n_cat(self) -> int:
        return _up(self.heads_out + self.w + self.f, 128)


@dataclass
class KabanexLayerWeights:
    norm_w: torch.Tensor     # f32
    norm_b: torch.Tensor
    w_in: object             # [n_mix + f, d]   (TiledWeight on a bf16 GPU model)
    w_out: object            # [hidden padded to 16, n_cat]
    talk: torch.Tensor       # f32 [H, H]
    talk_frag: Optional[torch.Tensor]  # the same as the prefill kernel's A operand (None: too many heads for it)
    zb: torch.Tensor         # f32 [width]
    xb: torch.Tensor


class KabanexModel:
    stateful = True          # recurrent state per sequence: prefix-cached blocks alone cannot resume one
    shared_buffers = ("talk",)   # step buffers that ragged forwards use as well

    def __init__(self, cfg: KabanexConfig, *, device="cpu", dtype: Optional[torch.dtype] = None,
                 tp: Optional[TPContext] = None, seed: int = 0, weights: Optional[dict] = None):
        self.cfg = cfg
        self.device = torch.device(device)
        self.dtype = dtype or (torch.bfloat16 if self.device.type == "cuda" else torch.float32)
        if self.dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"unsupported dtype {self.dtype} (bfloat16 | float32)")
        self.tp = tp or TPContext.single()
        assert self.tp.size == 1, "Kabanex runs on one GPU"
        self.dims: List[LayerDims] = [LayerDims.of(cfg, L) for L in cfg.layers]
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
        cfg, dev, dt = self.cfg, self.device, self.dtype
        tiled = dev.type == "cuda" and dt == torch.bfloat16
        place = (lambda t: ops.TiledWeight(t)) if tiled else (lambda t: t)
        vec = lambda n: w[n].to(device=dev, dtype=torch.float32).contiguous()  # noqa: E731

        def mat(name, rows, cols):
            t = w[name]
            if tuple(t.shape) != (rows, cols):
                raise ValueError(f"{name}: shape {tuple(t.shape)}, expected {(rows, cols)}")
            return t.to(device=dev, dtype=dt)

        self.embed = mat("embed", cfg.vocab_size, cfg.hidden).contiguous()
        self.layers: List[KabanexLayerWeights] = []
        for i, (L, D) in enumerate(zip(cfg.layers, self.dims)):
            a, W, d = L.left, L.right.width, cfg.hidden
            p = f"l{i}."
            w_in = torch.zeros(D.n_mix + D.f, D.d, dtype=dt, device=dev)
            k0, v0, g0, z0, x0, r0 = D.at

            def heads(at, name, n, size, pad):
                w_in[at : at + n * pad].view(n, pad, D.d)[:, :size, :d] = mat(name, n * size, d).view(n, size, d)

            heads(0, p + "mix.left.q", a.heads, a.dim, D.dk)
            heads(k0, p + "mix.left.k", a.kv_heads, a.dim, D.dk)
            heads(v0, p + "mix.left.v", a.kv_heads, a.vdim, D.dv)
            w_in[g0 : g0 + a.heads, :d] = mat(p + "mix.left.g", a.heads, d)
            for at, name in ((z0, "z"), (x0, "x"), (r0, "g")):
                w_in[at : at + W, :d] = mat(p + "mix.right." + name, W, d)
            w_out = torch.zeros(self.n_out, D.n_cat, dtype=dt, device=dev)
            o = mat(p + "mix.left.o", d, a.heads * a.vdim).view(d, a.heads, a.vdim)
            w_out[:d, : D.heads_out].view(d, D.H, D.dv)[:, :, : a.vdim] = o
            w_out[:d, D.heads_out : D.heads_out + W] = mat(p + "mix.right.o", d, W)
            if L.ffn:
                w_in[D.n_mix : D.n_mix + L.ffn, :d] = mat(p + "mlp.up", L.ffn, d)
                at = D.heads_out + D.w
                w_out[:d, at : at + L.ffn] = mat(p + "mlp.down", d, L.ffn)
            talk = vec(p + "mix.left.talk")
            if tuple(talk.shape) != (a.heads, a.heads):
                raise ValueError(f"{p}mix.left.talk: shape {tuple(talk.shape)}, expected {(a.heads, a.heads)}")
            self.layers.append(KabanexLayerWeights(
                norm_w=vec(p + "norm1"), norm_b=vec(p + "norm1.b"), w_in=place(w_in), w_out=place(w_out), talk=talk,
                talk_frag=ops.talk_fragment(talk, a.kv_heads) if tiled and _padded_heads(a) <= 32 else None, zb=vec(p + "mix.right.z.b"), xb=vec(p + "mix.right.x.b")))
        self.final_w, self.final_b = vec("final.norm"), vec("final.norm.b")
        head = torch.zeros(self.v_pad, self.d_pad, dtype=dt, device=dev)
        head[: cfg.vocab_size, : cfg.hidden] = mat("head", cfg.vocab_size, cfg.hidden)
        self.lm_head = place(head)

    def weight_bytes(self) -> int:
        ts = [self.lm_head] + [t for L in self.layers for t in (L.w_in, L.w_out)]
        return sum(t.numel() * t.element_size() for t in ts)

    # ------------------------------------------------------------------ engine hooks
    def ensure_positions(self, n: int) -> None:
        """Rotation tables (one per distinct base and size) for at least n positions."""
        for L in self.cfg.layers:
            key = (L.left.rot_base, L.left.rot_dims)
            t = self.ropes.get(key)
            if t is None or t.shape[0] < n:
                if t is not None:
                    self._old_ropes.append(t)  # (another engine's captured graphs may hold its address)
                self.ropes[key] = ops.rope_table(n, key[1], key[0], device=self.device)

    def cache_layers(self) -> List[CacheLayer]:
        return [CacheLayer(n_kv_heads=D.G, k_dim=D.dk, v_dim=D.dv, v_transposed=True, state=L.right.width)
                for L, D in zip(self.cfg.layers, self.dims)]

    def row_buffers(self, rows: int, max_ctx: int) -> Dict[str, object]:
        """Activation buffers of a step of ``rows`` rows (fixed addresses when the engine keeps them)."""
        dev, dt = self.device, self.dtype
        e = lambda *n, t=dt: torch.empty(*n, dtype=t, device=dev)  # noqa: E731
        # every buffer is written before it is read, but for the padding columns of a concatenation row: zeroed
        # once, never written (so each distinct layout has rows of its own)
        full = {D: D.n_cat == D.heads_out + L.right.width + L.ffn for L, D in zip(self.cfg.layers, self.dims)}
        return dict(hidden=e(rows, self.d_pad, t=torch.float32), normed=e(rows, self.d_pad),
                    mix=e(rows * max(D.n_mix for D in self.dims)), q=e(rows * max(D.H * D.dk for D in self.dims)),
                    cat={D: e(rows, D.n_cat) if ok else torch.zeros(rows, D.n_cat, dtype=dt, device=dev)
                         for D, ok in full.items()})

    def step_buffers(self, rows: int, max_ctx: int) -> Dict[str, object]:
        dev = self.device
        b = self.row_buffers(rows, max_ctx)
        b.update(hidden_sel=torch.zeros(rows, self.d_pad, dtype=torch.float32, device=dev),
                 head_in=torch.zeros(rows, self.d_pad, dtype=self.dtype, device=dev),
                 logits_local=torch.zeros(rows, self.v_pad, dtype=torch.float32, device=dev),
                 talk=ops.TalkScratch([(D.H, D.G, D.dv, L.left.window, L.left.keep_first)
                                       for L, D in zip(self.cfg.layers, self.dims)], max_ctx, dev))
        return b

    def plan_rows(self, runs: Sequence[Tuple[int, int, int, int]], max_pos: int) -> SimpleNamespace:
        return ops.plan_runs(runs, self.device, max_pos)

    # ------------------------------------------------------------------ forward
    def forward(self, bufs, M: int, kv, *, n_sel: Optional[int] = None, head: bool = True) -> torch.Tensor:
        """M ragged rows (bufs: tokens, positions, seq_ids, slots; ``plan`` for prompt-sized steps) ->
        f32 logits, or the residual rows with head=False (all, or those in bufs.sel[:n_sel])."""
        x = bufs.hidden[:M]
        plan = getattr(bufs, "plan", None)
        rows = dict(positions=bufs.positions[:M], seq_ids=bufs.seq_ids[:M], slots=bufs.slots[:M])
        ops.embedding_f32(bufs.tokens[:M], self.embed, out=x)
        h = bufs.normed[:M]
        for li in range(self.cfg.n_layers):
            self._layer(li, bufs, M, kv, x, h, rows, plan)
        if n_sel is not None:
            x = torch.index_select(x, 0, bufs.sel[:n_sel], out=bufs.hidden_sel[:n_sel])
        return self.lm_logits(bufs, x) if head else x

    def _layer(self, li: int, bufs, M: int, kv, x, h, rows, plan) -> None:
        C, D, L = self.cfg.layers[li], self.dims[li], self.layers[li]
        a = C.left
        _, _, g0, z0, x0, r0 = D.at
        ops.layernorm_f32(x, L.norm_w, L.norm_b, eps=self.cfg.norm_eps, out=h)
        y = bufs.mix[: M * D.n_mix].view(M, D.n_mix)
        cat = bufs.cat[D][:M]
        r_at, f_at = D.heads_out, D.heads_out + D.w
        ops.linear_split(h, L.w_in, y, cat[:, f_at : f_at + D.f] if D.f else None)
        W = C.right.width
        q = ops.qkv_cache_mingru(y, (z0, x0, r0), L.zb, L.xb, n_q_heads=D.H, rot_dims=a.rot_dims,
                                 rope=self.ropes[(a.rot_base, a.rot_dims)], q_out=bufs.q[: M * D.H * D.dk].view(M, D.H * D.dk),
                                 k_cache=kv.k[li], v_cache=kv.v[li], state=kv.state[li], out_scale=C.right_scale,
                                 out=cat[:, r_at : r_at + W], plan=plan, **rows)
        ops.talk_attention(q, kv.k[li], kv.v[li], bufs.block_table, n_q_heads=D.H, scale=a.scale, window=a.window,
                           keep=a.keep_first, talk=L.talk, talk_frag=L.talk_frag, gate=y[:, g0 : g0 + D.gate],
                           out_scale=C.left_scale, max_ctx=bufs.max_ctx, scratch=bufs.talk, out=cat[:, : D.heads_out],
                           plan=plan, **rows)
        xo = x[:, : self.n_out]
        ops.linear(cat, L.w_out, out=xo, residual=xo)

    def lm_logits(self, bufs, hs: torch.Tensor, col_mask: Optional[torch.Tensor] = None, mask_rows: int = 1,
                  gather: bool = True) -> torch.Tensor:
        """Final LayerNorm + LM head of residual rows -> f32 logits [rows, vocab] (contract as
        LlamaModel.lm_logits)."""
        n = hs.shape[0]
        fits = n <= bufs.logits_local.shape[0]
        h = bufs.head_in[:n] if fits else torch.empty(n, self.d_pad, dtype=self.dtype, device=hs.device)
        out = bufs.logits_local[:n] if fits else torch.empty(n, self.v_pad, dtype=torch.float32, device=hs.device)
        ops.layernorm_f32(hs, self.final_w, self.final_b, eps=self.cfg.norm_eps, out=h)
        if col_mask is not None and (self.dtype != torch.bfloat16 or col_mask.shape[1] * 32 < self.v_pad):
            col_mask = None
        ops.linear(h, self.lm_head, out=out, out_dtype=torch.float32, col_mask=col_mask, mask_rows=mask_rows)
        return out[:, : self.cfg.vocab_size]


class _RandomWeights:
    """Random tensors under the checkpoint's names, made on access (deterministic per name)."""

    def __init__(self, cfg: KabanexConfig, seed: int, device):
        self.cfg, self.seed, self.device = cfg, seed, device
        self.shapes = {}
        d, s = cfg.hidden, self.shapes
        s["embed"] = s["head"] = (cfg.vocab_size, d)
        s["final.norm"] = s["final.norm.b"] = (d,)
        for i, L in enumerate(cfg.layers):
            a, W, p = L.left, L.right.width, f"l{i}."
            s[p + "norm1"] = s[p + "norm1.b"] = (d,)
            m = p + "mix."
            s.update({m + "left.q": (a.heads * a.dim, d), m + "left.k": (a.kv_heads * a.dim, d),
                      m + "left.v": (a.kv_heads * a.vdim, d), m + "left.talk": (a.heads, a.heads),
                      m + "left.g": (a.heads, d), m + "left.o": (d, a.heads * a.vdim), m + "right.z": (W, d),
                      m + "right.z.b": (W,), m + "right.x": (W, d), m + "right.x.b": (W,), m + "right.g": (W, d),
                      m + "right.o": (d, W)})
            if L.ffn:
                s.update({p + "mlp.up": (L.ffn, d), p + "mlp.down": (d, L.ffn)})

    def __getitem__(self, name: str) -> torch.Tensor:
        shape = self.shapes[name]
        gen = torch.Generator(device=self.device)
        gen.manual_seed(self.seed * 1000003 + sum(ord(c) * 131 ** (i % 8) for i, c in enumerate(name)) % (1 << 31))
        t = torch.empty(shape, device=self.device, dtype=torch.float32).normal_(0.0, self.cfg.init_std, generator=gen)
        if name.endswith(("norm", "norm1")):
            t += 1.0
        elif name.endswith("talk"):  # near the identity, as a trained mixing would start
            t += torch.eye(shape[0], device=self.device)
        return t
