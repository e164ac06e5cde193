"""Ops of layer stacks with an f32 residual stream (csrc/kernels/stack_ops.hip, talk_attention.hip,
recurrence.hip, gemm_f32.hip): activations, caches and weights are bf16, or 32-bit for models that
run in 32-bit; norms, scores, softmax weights, recurrent state and the residual are f32 either way.

Cache layout of these ops: K ``[blocks, kv_heads, block_size, dk]``, V transposed inside a block,
``[blocks, kv_heads, dv, block_size]`` (the MFMA A-operand order of V^T).  ``dk`` is a multiple of 32
and ``dv`` of 16; the models pad smaller heads with zero weight rows.
"""
from __future__ import annotations

from types import SimpleNamespace
from typing import List, Optional, Sequence, Tuple

import torch

from . import reference as ref

TILE_ROWS = 16      # queries per workgroup of the prefill attention
SCAN_ROWS = 32      # rows per chunk of the recurrence scan
ROW_SLICE = 64      # rows per launch of the rows-form attention (its scratch is sized for them)


def _ext():
    from . import ext

    return ext()


# ----------------------------------------------------------------------------- row plans
def plan_runs(runs: Sequence[Tuple[int, int]], device, max_pos: int, scan_rows: int = SCAN_ROWS) -> SimpleNamespace:
    """Launch tables of a ragged step with many rows.  runs: (first row, rows, ..), each of one sequence at
    consecutive positions; max_pos: the largest position of the step.  tiles: prefill attention tiles of the runs longer than one row; singles:
    the rows that are a run of their own (decoded tokens beside prompt portions); chunks: recurrence
    scan chunks (of scan_rows rows) of every run."""
    tiles: List[List[int]] = []
    singles: List[int] = []
    chunks: List[List[int]] = []
    for r0, n, *_ in runs:
        if n == 1:
            singles.append(r0)
        else:
            tiles += [[r0 + i, min(TILE_ROWS, n - i)] for i in range(0, n, TILE_ROWS)]
        k = -(-n // scan_rows)
        chunks += [[r0 + i * scan_rows, min(scan_rows, n - i * scan_rows), i, k] for i in range(k)]

    def dev(x, cols):
        t = torch.tensor(x, dtype=torch.int32).view(-1, cols)
        return t.pin_memory().to(device, non_blocking=True) if torch.device(device).type == "cuda" else t

    return SimpleNamespace(max_pos=max_pos, tiles=dev(tiles, 2) if tiles else None, chunks=dev(chunks, 4),
                           singles=dev(singles, 1).view(-1) if singles else None)


def visible_tiles(max_ctx: int, window: int, keep: int) -> int:
    """16-key tiles a row can see at most."""
    tiles = -(-max_ctx // 16)
    return min(tiles, -(-keep // 16) + (window + 14) // 16 + 1) if window > 0 else tiles


def visible_chunks(max_ctx: int, window: int, keep: int) -> int:
    """128-key chunks a row can see at most: sizes the rows-form scratch."""
    return -(-visible_tiles(max_ctx, window, keep) // 8)


class TalkScratch:
    """Score / statistics / partial buffers of the rows-form attention for ROW_SLICE rows, sized for the
    largest layer (fixed addresses: captured step graphs use them)."""

    def __init__(self, layers: Sequence[Tuple[int, int, int, int, int]], max_ctx: int, device):
        """layers: (query heads, kv heads, dv, window, keep) of every layer."""
        s = stat = part = cnt = 1
        for H, G, dv, window, keep in layers:
            n = visible_chunks(max_ctx, window, keep)
            s, stat = max(s, H * n * 128), max(stat, H * n * 2)
            part, cnt = max(part, n * H * dv), max(cnt, G * -(-(H // G) // 16))
        f32 = dict(dtype=torch.float32, device=device)
        self.s = torch.zeros(ROW_SLICE * s, **f32)
        self.stat = torch.zeros(ROW_SLICE * stat, **f32)
        self.part = torch.zeros(ROW_SLICE * part, **f32)
        self.counters = torch.zeros(ROW_SLICE * cnt, dtype=torch.int32, device=device)


# ----------------------------------------------------------------------------- ops
def layernorm_f32(x: torch.Tensor, w: torch.Tensor, b: Optional[torch.Tensor], *, eps: float, out: torch.Tensor) -> torch.Tensor:
    """out = (x - mean) / sqrt(var + eps) * w (+ b) of f32 rows; out may be wider than w (zero columns)."""
    if not x.is_cuda:
        return ref.layernorm_f32(x, w, b, eps=eps, out=out)
    _ext().layernorm_f32(x, w, b, out, eps)
    return out


def add_norm(x: torch.Tensor, branch: torch.Tensor, w1: torch.Tensor, w2: Optional[torch.Tensor], *, eps: float,
             out: Optional[torch.Tensor] = None, n_parts: int = 1) -> None:
    """The end of a sublayer and the start of the next: x (f32 rows) += norm(branch) * w1, out = norm(x) * w2
    (w2 None: not computed).  branch rows n_parts * i .. are added up for row i; layer norms without bias."""
    if not x.is_cuda:
        return ref.add_norm(x, branch, w1, w2, eps=eps, out=out, n_parts=n_parts)
    _ext().add_norm(x, branch, n_parts, w1, w2, out, eps)


def embedding_f32(ids: torch.Tensor, table: torch.Tensor, *, out: torch.Tensor, scale: float = 1.0) -> torch.Tensor:
    """f32 residual rows from the embedding table, scaled; out may be wider than the table (zero columns)."""
    if not out.is_cuda:
        return ref.embedding_f32(ids, table, out=out, scale=scale)
    _ext().embedding_f32(ids, table, out, scale)
    return out


def linear_split(x: torch.Tensor, w, out: torch.Tensor, out2: Optional[torch.Tensor]) -> torch.Tensor:
    """One projection of a normed row for a layer's mixers and its feed-forward: the first out.shape[1]
    columns of x @ w^T to ``out``, relu(.)^2 of the others to ``out2`` (None: there are none)."""
    from . import SKINNY_MAX_M, TiledWeight, GEMM_WS_FLOATS, linear, scratch

    if out2 is None:
        return linear(x, w, out=out)
    if not x.is_cuda:
        return ref.linear_split(x, w, out=out, out2=out2)
    if x.dtype == torch.float32:
        _ext().gemm_f32(x, w, out, 6, None, out2)
        return out
    tiled = isinstance(w, TiledWeight)
    wt = w.t if tiled else w
    if x.shape[0] <= SKINNY_MAX_M and tiled:
        _ext().skinny_gemm(x, wt, None, out, 5, False, 0.0, None, None, None, True, y2=out2)
    else:
        _ext().gemm(x, wt, None, out, 6, None, None, tiled, scratch(x.device, "gemm_ws", GEMM_WS_FLOATS), y2=out2)
    return out


def qkv_cache_write(x: torch.Tensor, *, n_q_heads: int, rot_dims: int, rope: torch.Tensor, positions: torch.Tensor,
                    slots: torch.Tensor, q_out: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor) -> torch.Tensor:
    """Rows [q | k | v]: rotate the first rot_dims dimensions of the q / k heads, q to q_out, k and v to
    the paged cache (slot < 0: not written)."""
    G, dk, dv = k_cache.shape[1], k_cache.shape[3], v_cache.shape[2]
    if not x.is_cuda:
        return ref.qkv_cache_write(x, n_q_heads=n_q_heads, rot_dims=rot_dims, rope=rope, positions=positions, slots=slots,
                                   q_out=q_out, k_cache=k_cache, v_cache=v_cache)
    _ext().qkv_cache(x, n_q_heads, G, dk, dv, rot_dims, rope, positions, slots, q_out, k_cache, v_cache)
    return q_out


def qkv_cache_mingru(y: torch.Tensor, at: Tuple[int, int, int], zb: torch.Tensor, xb: torch.Tensor, *, n_q_heads: int,
                     rot_dims: int, rope: torch.Tensor, positions: torch.Tensor, seq_ids: torch.Tensor, slots: torch.Tensor,
                     q_out: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, state: torch.Tensor,
                     out_scale: float, out: torch.Tensor, plan: Optional[SimpleNamespace] = None) -> torch.Tensor:
    """qkv_cache_write of a layer's projected rows and the mingru of its columns at = (z, x, g): one launch
    for a decode step on the GPU, else the two ops."""
    W = state.shape[1]
    z, x, g = (y[:, a : a + W] for a in at)
    if y.is_cuda and plan is None:
        G, dk, dv = k_cache.shape[1], k_cache.shape[3], v_cache.shape[2]
        _ext().qkv_mingru(y, n_q_heads, G, dk, dv, rot_dims, rope, positions, slots, q_out, k_cache, v_cache, z, x, g, zb, xb,
                          seq_ids, state, out_scale, out)
        return q_out
    qkv_cache_write(y, n_q_heads=n_q_heads, rot_dims=rot_dims, rope=rope, positions=positions, slots=slots, q_out=q_out,
                    k_cache=k_cache, v_cache=v_cache)
    mingru(z, x, g, zb, xb, seq_ids=seq_ids, positions=positions, slots=slots, state=state, out_scale=out_scale, out=out,
           plan=plan)
    return q_out


def talk_attention(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor, block_table: torch.Tensor,
                   positions: torch.Tensor, seq_ids: torch.Tensor, slots: torch.Tensor, *, n_q_heads: int, scale: float,
                   window: int, keep: int, talk: Optional[torch.Tensor], talk_frag: Optional[torch.Tensor],
                   gate: Optional[torch.Tensor], out_scale: float, max_ctx: int, scratch: Optional[TalkScratch],
                   out: torch.Tensor, plan: Optional[SimpleNamespace] = None) -> torch.Tensor:
    """Attention of ragged rows over their sequences' cached keys: row i sees key j if j <= i and
    (i - j < window or j < keep) (window 0: every key); softmax weights mixed across heads by ``talk``
    [H, H] (None: not mixed), heads gated by sigmoid(gate), the result scaled by out_scale.
    plan (plan_runs): prompt-sized steps -- runs go to the MFMA prefill form where it takes the sizes,
    single rows and everything else to the rows form."""
    if not q.is_cuda:
        return ref.talk_attention(q, k_cache, v_cache, block_table, positions, seq_ids, slots, n_q_heads=n_q_heads,
                                  scale=scale, window=window, keep=keep, talk=talk, gate=gate, out_scale=out_scale, out=out)
    E, rows = _ext(), q.shape[0]

    def rows_form(qs, pos, sid, slt, gt, o, row_list, n):
        E.talk_attention(qs, k_cache, v_cache, block_table, pos, sid, slt, row_list, n, n_q_heads, scale, window, keep, talk,
                         gt, out_scale, max_ctx, scratch.s, scratch.stat, scratch.part, scratch.counters, o)

    G, dk, dv = k_cache.shape[1], k_cache.shape[3], v_cache.shape[2]
    part = E.talk_prefill_part(n_q_heads, G, dk, dv) if plan is not None and talk_frag is not None else -1
    if part > 0 and q.dtype == torch.bfloat16 and visible_tiles(max_ctx, window + 15 if window > 0 else 0, keep) <= 1024:
        if plan.tiles is not None:
            from . import scratch as ws

            nt = plan.tiles.shape[0]
            splits = prefill_splits(nt, plan.max_pos, window, keep, E.device_cus(q))
            E.talk_prefill(q, k_cache, v_cache, block_table, positions, seq_ids, slots, plan.tiles, n_q_heads, scale, window,
                           keep, talk_frag, gate, out_scale, max_ctx, splits, ws(q.device, "talk_lse", rows * n_q_heads),
                           ws(q.device, "talk_part", nt * splits * part if splits > 1 else 1), _tickets(q.device, nt), out)
        if plan.singles is not None:
            n = plan.singles.shape[0]
            for i in range(0, n, ROW_SLICE):
                lst = plan.singles[i : min(n, i + ROW_SLICE)]
                rows_form(q, positions, seq_ids, slots, gate, out, lst, lst.shape[0])
        return out
    for i in range(0, rows, ROW_SLICE):
        j = min(rows, i + ROW_SLICE)
        rows_form(q[i:j], positions[i:j], seq_ids[i:j], slots[i:j], None if gate is None else gate[i:j], out[i:j], None, j - i)
    return out


def prefill_splits(n_tiles: int, max_pos: int, window: int, keep: int, cus: int) -> int:
    """Workgroups per 16-query tile over its keys: enough to give every CU one, and no more than leaves
    each a round of its waves (128 keys)."""
    keys = max_pos + 1
    if window > 0:
        keys = min(keys, window + keep + 2 * TILE_ROWS)
    return max(1, min(-(-keys // 128), cus // n_tiles))


_TICKETS: dict = {}


def _tickets(device, n: int) -> torch.Tensor:
    """Zeroed chunk tickets of the prefill form (the kernel leaves them zero)."""
    t = _TICKETS.get(str(device))
    if t is None or t.numel() < n:
        t = _TICKETS[str(device)] = torch.zeros(max(n, 4096), dtype=torch.int32, device=device)
    return t


def talk_fragment(talk: torch.Tensor, n_kv_heads: int) -> torch.Tensor:
    """talk [H, H] as the prefill kernel's A operand (stack_kernels.h TalkPrefillParams::talk_frag), in its
    padded head order h = c * RP + r (kv heads and query heads per kv head rounded up to powers of two)."""
    H = talk.shape[0]
    R = H // n_kv_heads
    up = lambda n: 1 << (n - 1).bit_length()  # noqa: E731
    GP, RP = up(n_kv_heads), up(R)
    HT = GP * RP
    idx = torch.tensor([(h // R) * RP + h % R for h in range(H)])
    rows, cols = max(16, -(-HT // 16) * 16), max(HT, 4)
    T = torch.zeros(rows, cols)
    T[idx[:, None], idx[None, :]] = talk.detach().float().cpu()
    k = torch.arange(32)
    head = k % max(HT, 4) if HT < 32 else k
    live = k < 2 * max(HT, 4)                    # (hi and lo halves of the weights share the matrix)
    A = T[:, head] * live                        # [rows, 32]
    if HT > 32:
        raise ValueError(f"{HT} padded heads: the prefill kernel takes 32")
    A = A.view(rows // 16, 16, 4, 8).permute(0, 2, 1, 3)   # [mt][lane group b][row rl][e]
    return A.reshape(rows // 16, 64, 8).contiguous().to(device=talk.device, dtype=torch.bfloat16)


def mingru(z: torch.Tensor, x: torch.Tensor, g: torch.Tensor, zb: Optional[torch.Tensor], xb: Optional[torch.Tensor], *,
           seq_ids: torch.Tensor, positions: torch.Tensor, slots: torch.Tensor, state: torch.Tensor, out_scale: float,
           out: torch.Tensor, plan: Optional[SimpleNamespace] = None) -> torch.Tensor:
    """Gated recurrence over ragged rows: S <- (1 - z) S + z cand, out = S * silu(g) * out_scale; the state
    row of a sequence is its id, read and written once per run (position 0 starts from zero)."""
    if not z.is_cuda:
        return ref.mingru(z, x, g, zb, xb, seq_ids=seq_ids, positions=positions, slots=slots, state=state,
                          out_scale=out_scale, out=out)
    from . import scratch

    if plan is None:
        _ext().mingru(z, x, g, zb, xb, seq_ids, positions, slots, state, out_scale, out)
    else:
        n = 3 * plan.chunks.shape[0] * state.shape[1]
        _ext().mingru(z, x, g, zb, xb, seq_ids, positions, slots, state, out_scale, out, plan.chunks,
                      scratch(z.device, "scan", n))
    return out
