"""Mixers and feed-forwards of serial layer stacks (csrc/kernels/rglru.hip, latent.hip, moe.hip): the
real-gated linear recurrence behind a short convolution, latent attention, routed experts.

Activations, caches and weights are bf16, or 32-bit for models that run in 32-bit; scores, softmax
weights, norms, router scores, gates of the recurrence and its state are f32 either way.  Sizes are
padded by the models with zero weight rows / columns: blocks of recurrence channels, head sizes and
the latent to 32, values to 16.

Cache row of a token: ``[latent (rank_p) | rotated key part (rot_p)]`` in pages
``[blocks, 1, block_size, rank_p + rot_p]``; state row of a sequence: ``[S | last taps - 1 inputs]``.
"""
from __future__ import annotations

from dataclasses import dataclass
from types import SimpleNamespace
from typing import Optional, Sequence, Tuple

import torch

from . import reference as ref
from .stack import ROW_SLICE, _ext

SCAN_ROWS = 64      # rows per chunk of the recurrence scan
ATTN_KEYS = 64      # keys per round of the latent attention
ATTN_GROUPS = 512   # workgroups a latent attention launch is cut into
EXPAND_ROWS = 32    # runs of fewer rows attend in latent space ...
EXPAND_CONTEXT = 128  # ... and so do runs behind more than this many tokens of context per row
MOE_TILES = (16, 32, 128, 256)  # pairs per tile of the experts' products: streaming kernel, LDS-tiled GEMM


# ----------------------------------------------------------------------------- weight layouts
def fragments(w: torch.Tensor) -> torch.Tensor:
    """w [.., N, K] (N a multiple of 16, K of 32) in MFMA operand order (mixer_kernels.h "fragment order"):
    [.., N / 16, K / (4 EPL), 64 lanes, EPL], flattened; EPL = 8 bf16 / 4 floats."""
    epl = 16 // w.element_size()
    *b, N, K = w.shape
    t = w.reshape(*b, N // 16, 16, K // (4 * epl), 4, epl)
    return t.movedim(-4, -2).contiguous().view(-1)                      # [.., T, step, g, n, e]


def tile_weights(w: torch.Tensor) -> torch.Tensor:
    """w [E, N, K] pre-tiled per matrix as ops.tile_weight (f32: the same order with 4-element pieces)."""
    epl = 16 // w.element_size()
    E, N, K = w.shape
    t = w.reshape(E, N // 16, 16, K // (16 * epl), 4, 4, epl)           # [E, T, n, kg, g, s, e]
    return t.permute(0, 1, 3, 5, 4, 2, 6).contiguous().view(E, N, K)    # [E, T, kg, s, g, n, e]


# ----------------------------------------------------------------------------- recurrence
@dataclass
class RgLruWeights:
    """Padded per block (nb blocks of bs channels).  gates: [nb, 2 (r, i), bs, bs], as fragments on a GPU."""
    nb: int
    yb: torch.Tensor
    xb: torch.Tensor
    conv: torch.Tensor       # f32 [taps, width], last row: the current token
    conv_b: torch.Tensor
    gates: torch.Tensor
    rb: torch.Tensor
    ib: torch.Tensor
    decay: torch.Tensor      # f32 [width]: -8 softplus(lam)


def gate_fragments(gates: torch.Tensor) -> torch.Tensor:
    """[nb, 2, bs, bs] -> [nb][16-channel tile][r, i][steps][64][EPL]."""
    nb, _, bs, _ = gates.shape
    f = fragments(gates).view(nb, 2, bs // 16, -1)
    return f.transpose(1, 2).contiguous().view(-1)


def rglru(yx: torch.Tensor, w: RgLruWeights, *, seq_ids: torch.Tensor, positions: torch.Tensor, slots: torch.Tensor,
          state: torch.Tensor, out: torch.Tensor, plan: Optional[SimpleNamespace] = None) -> torch.Tensor:
    """yx rows [y | x] (raw projections): u = causal conv of x + its bias, r / i from u block by block,
    S <- a S + sqrt(1 - a^2) i u with log a = decay r, out = S gelu_tanh(y + bias).  The state row of a
    sequence is its id, read and written once per run (position 0 starts from zeros)."""
    if not yx.is_cuda:
        return ref.rglru(yx, w, seq_ids=seq_ids, positions=positions, slots=slots, state=state, out=out)
    args = (yx, w.yb, w.xb, w.conv, w.conv_b, w.gates, w.rb, w.ib, w.decay, w.nb, seq_ids, positions, slots, state, out)
    if plan is None:
        _ext().rglru(*args)
    else:
        from . import scratch

        W = w.decay.numel()
        _ext().rglru(*args, plan.chunks, scratch(yx.device, "scan", 3 * plan.chunks.shape[0] * W),
                     scratch(yx.device, "rglru_u", out.shape[0] * W, yx.dtype))
    return out


# ----------------------------------------------------------------------------- latent attention
@dataclass
class LatentWeights:
    """uk [H, rank_p, dim_p] (keys' projection, transposed), uv [H, vd, rank_p]: as fragments on a GPU."""
    H: int
    dim_p: int
    rot_p: int
    rank_p: int
    vd: int
    scale: float
    eps: float
    norm: Optional[torch.Tensor]   # f32 [rank]; None: another layer's latent
    sink: torch.Tensor             # f32 [H]
    uk: torch.Tensor
    uv: torch.Tensor
    w_kv: object = None            # prompts: the keys' and values' projections [H (dim_p + vdk), rank to 128] (TiledWeight)

    @property
    def vdk(self) -> int:
        """Value columns of a head in the expanded rows."""
        return -(-self.vd // 32) * 32


def latent_chunks(rows: int, H: int, max_ctx: int) -> int:
    """Key chunks per row of a launch over ``rows`` rows."""
    return max(1, min(-(-max_ctx // ATTN_KEYS), ATTN_GROUPS // (rows * -(-H // 16))))


class LatentScratch:
    """Partial sums and statistics of the rows-form attention for up to ROW_SLICE rows, sized for the largest
    layer (fixed addresses: captured step graphs use them)."""

    def __init__(self, layers: Sequence[Tuple[int, int]], max_ctx: int, device):
        """layers: (heads, rank_p) of every layer."""
        part = stat = 1
        for H, rank_p in layers:
            n = max(r * latent_chunks(r, H, max_ctx) for r in range(1, ROW_SLICE + 1))
            part, stat = max(part, n * H * rank_p), max(stat, n * H * 2)
        self.part = torch.zeros(part, dtype=torch.float32, device=device)
        self.stat = torch.zeros(stat, dtype=torch.float32, device=device)


def plan_latent(runs: Sequence[Tuple[int, int, int, int]], device, plan: SimpleNamespace) -> SimpleNamespace:
    """Attention tables of a ragged step, added to ``plan``.  runs: (first row, rows, block-table row, first
    position).  Runs worth expanding their context go to the prefill form: q_tiles (the longest contexts
    first) and segs (64 context rows each, one run after the other); short: the rows of the others."""
    tiles, segs, short = [], [], []
    for r0, n, sid, pos in runs:
        ctx = pos + n
        if n < EXPAND_ROWS or ctx > EXPAND_CONTEXT * n:
            short += range(r0, r0 + n)
            continue
        t0 = 64 * len(segs)
        segs += [[sid, k, ctx] for k in range(0, ctx, 64)]
        tiles += [[r0 + i, min(128, n - i), t0, pos + i] for i in range(0, n, 128)]
    tiles.sort(key=lambda t: -t[3])
    cuda = torch.device(device).type == "cuda"

    def dev(x, *shape):
        if not x:
            return None
        t = torch.tensor(x, dtype=torch.int32).view(*shape)
        return t.pin_memory().to(device, non_blocking=True) if cuda else t

    plan.q_tiles, plan.segs, plan.short = dev(tiles, -1, 4), dev(segs, -1, 3), dev(short, -1)
    return plan


def _expands(w: LatentWeights, y: torch.Tensor, plan) -> bool:
    """This step's long runs take the prefill form."""
    return (plan is not None and plan.q_tiles is not None and w.w_kv is not None and y.dtype == torch.bfloat16
            and _ext().latent_prefill_fits(w.dim_p, w.rot_p, w.vdk))


def latent_qkv(y: torch.Tensor, w: LatentWeights, *, rope: torch.Tensor, positions: torch.Tensor, slots: torch.Tensor,
               q_out: torch.Tensor, cache: Optional[torch.Tensor], plan: Optional[SimpleNamespace] = None) -> torch.Tensor:
    """Projected rows [q | latent | key part | ..]: the queries in latent space, rotated parts behind them
    (q_out [rows, H (rank_p + rot_p)]); latent normed, key part rotated, both to the cache (slot < 0: not
    written; ``cache`` None: the layer reads another layer's).  Rows of the prefill form get their rotated
    parts only."""
    if not y.is_cuda:
        return ref.latent_qkv(y, w, rope=rope, positions=positions, slots=slots, q_out=q_out, cache=cache)
    E, norm, dk, hq = _ext(), w.norm if cache is not None else None, w.rank_p + w.rot_p, w.dim_p + w.rot_p
    if not _expands(w, y, plan):
        E.latent_qkv(y, w.H, w.dim_p, w.rot_p, w.rank_p, rope, positions, slots, q_out, norm, w.eps, cache, w.uk)
        return q_out
    E.latent_rows(y, w.H, w.dim_p, w.rot_p, rope, positions, slots, q_out, dk, w.rank_p, norm, w.eps, cache)
    if plan.short is not None:
        E.head_linear(y, hq, w.uk, w.H, w.rank_p, w.dim_p, q_out, dk, plan.short)
    return q_out


def latent_attention(q: torch.Tensor, w: LatentWeights, *, cache: torch.Tensor, block_table: torch.Tensor, positions: torch.Tensor,
                     seq_ids: torch.Tensor, slots: torch.Tensor, gate: torch.Tensor, max_ctx: int, scratch: LatentScratch,
                     out: torch.Tensor, y: Optional[torch.Tensor] = None, plan: Optional[SimpleNamespace] = None) -> torch.Tensor:
    """Causal softmax with a sink per head over the cached latents, value projection, output gate.  y: the
    projected rows (the prefill form reads the unrotated query parts there)."""
    if not q.is_cuda:
        return ref.latent_attention(q, w, cache=cache, block_table=block_table, positions=positions, seq_ids=seq_ids,
                                    slots=slots, gate=gate, out=out)
    E, rows = _ext(), q.shape[0]

    def rows_form(row_list, i, n):
        nch = latent_chunks(n, w.H, max_ctx)
        s = slice(i, i + n) if row_list is None else slice(None)
        E.latent_attention(q[s], cache, block_table, positions[s], seq_ids[s], slots[s], row_list, n, w.H, w.rank_p, w.scale, nch,
                           scratch.part, scratch.stat)
        E.latent_out(scratch.part, scratch.stat, nch, slots[s], row_list, n, w.H, w.rank_p, w.sink, w.uv, gate[s], out[s])

    if y is None or not _expands(w, y, plan):
        for i in range(0, rows, ROW_SLICE):
            rows_form(None, i, min(ROW_SLICE, rows - i))
        return out
    if plan.short is not None:
        for i in range(0, plan.short.shape[0], ROW_SLICE):
            lst = plan.short[i : i + ROW_SLICE]
            rows_form(lst, 0, lst.shape[0])
    from . import linear, scratch as ws

    T, kp, n_kv, bf = 64 * plan.segs.shape[0], w.w_kv.shape[1], w.w_kv.shape[0], torch.bfloat16
    lat = ws(q.device, "latent_ctx", T * kp, bf).view(T, kp)
    krot = ws(q.device, "latent_rot", T * w.rot_p, bf).view(T, w.rot_p)
    kv = ws(q.device, "latent_kv", T * n_kv, bf).view(T, n_kv)
    E.latent_gather(cache, block_table, plan.segs, lat, krot)
    linear(lat, w.w_kv, out=kv)
    E.latent_prefill(y, q, w.H, w.dim_p, w.rank_p + w.rot_p, w.rank_p, kv[:, : w.H * (w.dim_p + w.vdk)], krot, plan.q_tiles, w.scale,
                     w.sink, gate, w.vd, out)
    return out


# ----------------------------------------------------------------------------- routed experts
@dataclass
class MoeWeights:
    """router [E padded to 16, K] (fragments on a GPU), gate_up [E, 2 F, K] (interleaved by 16), down [E, N, F]
    (pre-tiled on a GPU)."""
    E: int
    top: int
    router: torch.Tensor
    gate_up: torch.Tensor
    down: torch.Tensor


def moe_tiles(pairs: int, E: int, tile: int) -> int:
    """Most tiles that ``pairs`` pairs over E experts fill."""
    return min(pairs, E) + pairs // tile


def moe_tile(rows: int, E: int, top: int, dtype) -> int:
    """The tile size of a step: the larger streaming tile where many experts would fill two small ones, the
    LDS-tiled GEMM once its small tiles are a quarter full on average, its large ones once an expert fills one."""
    per = rows * top / E
    if dtype != torch.bfloat16 or per <= 8:
        return 16
    return 256 if per >= 256 else 128 if per >= 32 else 32


def moe_buffers(rows: int, layers: Sequence[Tuple[int, int, int]], dtype, device) -> SimpleNamespace:
    """Routing tables and expert activations of a step of up to ``rows`` rows; layers: (E, top, F) of every layer."""
    top = max(t for _, t, _ in layers)
    # (fewer rows may take the smaller tiles)
    sizes = [(moe_tiles(rows * t, E, tile), tile, f) for E, t, f in layers for tile in MOE_TILES if tile <= moe_tile(rows, E, t, dtype)]
    tiles = max(n for n, _, _ in sizes)
    places = max(n * t for n, t, _ in sizes)
    act = max(n * t * f for n, t, f in sizes)
    i32 = dict(dtype=torch.int32, device=device)
    return SimpleNamespace(wts=torch.zeros(rows * top, dtype=torch.float32, device=device), ids=torch.zeros(rows * top, **i32),
                           tiles=torch.zeros(1 + 3 * tiles, **i32), order=torch.zeros(places, **i32),
                           ticket=torch.zeros(1, **i32), act=torch.empty(act, dtype=dtype, device=device))


def moe(h: torch.Tensor, w: MoeWeights, *, slots: torch.Tensor, bufs: SimpleNamespace, out: torch.Tensor) -> torch.Tensor:
    """Every row's ``top`` best experts by sigmoid(router . h); out row (row * top + k) = expert_k(score h)."""
    rows = h.shape[0]
    if not h.is_cuda:
        return ref.moe(h, w, slots=slots, out=out)
    E, F, tile = _ext(), w.down.shape[2], moe_tile(rows, w.E, w.top, h.dtype)
    n = moe_tiles(rows * w.top, w.E, tile)
    tiles, order = bufs.tiles[: 1 + 3 * n], bufs.order[: n * tile]
    act = bufs.act[: n * tile * F].view(-1, F)
    E.moe_route(h, w.router, w.E, w.top, slots, bufs.wts, bufs.ids, tile, tiles, order, bufs.ticket)
    E.moe_gemm(h, w.gate_up, rows, w.top, False, bufs.wts, tile, tiles, order, act)
    E.moe_gemm(act, w.down, rows, w.top, True, bufs.wts, tile, tiles, order, out)
    return out
