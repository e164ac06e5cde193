// Windowed attention with kept first keys, mixed ("talking") heads and per-head output gates.
//
// Row i sees key j when j <= i and (i - j < window or j < keep).  With softmax weights w_g of query
// head g, head h applies sum_g talk[h][g] w_g to the values of its own kv head, so the weights of ALL
// heads for a key have to be normalised before any value is read: every form below computes the
// softmax statistics first and forms the (already normalised) mixed weights in a second pass.  The
// weights, their mixing and the statistics are f32; the mixed weights enter the value product as T.
//
// Keys are walked in 16-key tiles inside cache blocks.  The visible tiles of a row are those of the
// kept first keys, then those of the window (vis_tiles); edges are masked per key.
//
//  1) rows form (decode; any T, any sizes): launch A -- a workgroup per (row, kv head, 8 tiles)
//     computes S^T = K.Q^T on the MFMA (the kv head's query heads are the 16 columns), stores the
//     scores and the chunk's (max, sum) per head; launch B -- same grid -- folds the chunk statistics
//     of every head, mixes the chunk's weights into LDS in B-operand order and multiplies by V^T,
//     which the cache stores transposed (its A operand, no staging).  Chunks of a row are added in
//     chunk order by the last-arriving workgroup (sc1 hand-off + ticket, as decode attention).
//  2) prefill form (bf16), per 16 consecutive queries: launch A reduces the scores to log-sum-exps;
//     launch B recomputes them, a wave holding every head of its key tile, mixes the heads on the MFMA
//     and hands the mixed weights through LDS (B-operand order) to the waves' (kv head, 16 value
//     columns) tiles.
#include "common.h"
#include "mq_attention.h"
#include "stack_kernels.h"

using namespace vwa;

namespace {

constexpr int kTile = 16;                  // keys per tile
constexpr int kChunkTiles = 8;             // tiles per workgroup of the rows form
constexpr int kChunk = kTile * kChunkTiles;
constexpr float kLog2e = 1.4426950408889634f;

template <class T> struct MM;
template <> struct MM<u16> {               // 16-byte fragments: 8 k per lane, 32 per step
  static constexpr int KS = 32, EPL = 8;
  static VWA_DEVICE f32x4 mma(const uint4& a, const uint4& b, const f32x4& c) { return mfma16(as_bf16x8(a), as_bf16x8(b), c); }
};
template <> struct MM<float> {             // 4 k per lane, 16 per step: element j of every lane group per MFMA
  static constexpr int KS = 16, EPL = 4;
  static VWA_DEVICE f32x4 mma(const uint4& a, const uint4& b, f32x4 c) {
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.x), __uint_as_float(b.x), c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.y), __uint_as_float(b.y), c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.z), __uint_as_float(b.z), c, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.w), __uint_as_float(b.w), c, 0, 0, 0);
  }
};

template <class T> VWA_DEVICE float ldv(const T* p);
template <> VWA_DEVICE float ldv<u16>(const u16* p) { return bf2f(*p); }
template <> VWA_DEVICE float ldv<float>(const float* p) { return *p; }
VWA_DEVICE void stv(u16* p, float v) { *p = f2bf(v); }
VWA_DEVICE void stv(float* p, float v) { *p = v; }

struct Vis {
  int sink, first, n;                      // kept tiles 0 .. sink-1, then tiles first ..; n in all
};
// tiles seen by queries at positions p0 .. p1 together
VWA_DEVICE Vis vis_tiles(int p0, int p1, int window, int keep) {
  Vis v;
  v.first = window > 0 ? max(0, p0 - window + 1) / kTile : 0;
  v.sink = keep > 0 ? min((keep + kTile - 1) / kTile, v.first) : 0;
  v.n = v.sink + p1 / kTile - v.first + 1;
  return v;
}
VWA_DEVICE int tile_of(const Vis& v, int t) { return t < v.sink ? t : v.first + t - v.sink; }
VWA_DEVICE bool sees(int i, int j, int window, int keep) {
  return j <= i && (window <= 0 || i - j < window || j < keep);
}

// ------------------------------------------------------------------------------------------ rows form
template <class T>
__global__ __launch_bounds__(256) void talk_scores_kernel(TalkAttnParams p) {
  using M = MM<T>;
  __shared__ float sm[4][16][2];
  const int ri = blockIdx.x / p.G, c = blockIdx.x % p.G, chunk = blockIdx.y, r0 = blockIdx.z * 16;
  const int row = p.row_list ? p.row_list[ri] : ri;
  if (p.slots[row] < 0) return;
  const int pos = p.positions[row], seq = p.seq_ids[row];
  const Vis v = vis_tiles(pos, pos, p.window, p.keep);
  if (chunk * kChunkTiles >= v.n) return;
  const int R = p.H / p.G, Rb = min(16, R - r0);
  const int lane = lane_id(), w = threadIdx.x >> 6, rl = lane & 15, b = lane >> 4;
  const T* q = reinterpret_cast<const T*>(p.q) + (size_t)row * p.ldq + (size_t)(c * R + r0 + min(rl, Rb - 1)) * p.dk + b * M::EPL;
  const T* kp[2];
  int key0[2];
  bool ok[2];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int t = chunk * kChunkTiles + w * 2 + u;
    ok[u] = t < v.n;
    key0[u] = tile_of(v, ok[u] ? t : v.n - 1) * kTile;
    const int64_t blk = p.block_table[(int64_t)seq * p.table_stride + key0[u] / p.block_size];
    kp[u] = reinterpret_cast<const T*>(p.k) + blk * p.k_sb + (int64_t)c * p.k_sh +
            (int64_t)(key0[u] % p.block_size + rl) * p.dk + b * M::EPL;
  }
  f32x4 acc[2] = {};
#pragma unroll 4
  for (int k = 0; k < p.dk; k += M::KS) {
    const uint4 qf = *reinterpret_cast<const uint4*>(q + k);
#pragma unroll
    for (int u = 0; u < 2; ++u) acc[u] = M::mma(*reinterpret_cast<const uint4*>(kp[u] + k), qf, acc[u]);
  }
  // lane (column rl = head, keys 4b .. 4b+3 of both tiles): mask, store, chunk statistics
  float mx = -INFINITY;
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const bool vis = ok[u] && sees(pos, key0[u] + 4 * b + i, p.window, p.keep);
      acc[u][i] = vis ? acc[u][i] * p.scale : -INFINITY;
      mx = fmaxf(mx, acc[u][i]);
    }
  if (rl < Rb) {
#pragma unroll
    for (int u = 0; u < 2; ++u)
      if (ok[u])
        *reinterpret_cast<float4*>(p.s + ((size_t)ri * p.H + c * R + r0 + rl) * p.nch * kChunk +
                                   (chunk * kChunkTiles + w * 2 + u) * kTile + 4 * b) =
            make_float4(acc[u][0], acc[u][1], acc[u][2], acc[u][3]);
  }
  mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
  mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
  float l = 0.f;
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int i = 0; i < 4; ++i) l += acc[u][i] == -INFINITY ? 0.f : __expf(acc[u][i] - mx);
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (b == 0) {
    sm[w][rl][0] = mx;
    sm[w][rl][1] = l;
  }
  __syncthreads();
  if ((int)threadIdx.x < Rb) {
    const int r = threadIdx.x;
    float m = -INFINITY, s = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) m = fmaxf(m, sm[i][r][0]);
#pragma unroll
    for (int i = 0; i < 4; ++i) s += sm[i][r][1] > 0.f ? sm[i][r][1] * __expf(sm[i][r][0] - m) : 0.f;
    float* st = p.stat + (((size_t)ri * p.H + c * R + r0 + r) * p.nch + chunk) * 2;
    st[0] = m;
    st[1] = s;
  }
}

template <class T>
VWA_DEVICE float head_gate(const TalkAttnParams& p, int row, int h) {
  if (!p.gate) return p.out_scale;
  return p.out_scale / (1.f + __expf(-ldv(reinterpret_cast<const T*>(p.gate) + (size_t)row * p.ldg + h)));
}

// LDS: statistics [H][2], weights [H][128] f32, mixed weights [128 / KS][64][16 B]
template <class T>
size_t mix_lds(int H) { return (size_t)H * (2 + kChunk) * 4 + kChunk * 16 * sizeof(T); }

template <class T>
__global__ __launch_bounds__(256) void talk_mix_kernel(TalkAttnParams p) {
  using M = MM<T>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ int s_last;
  const int ri = blockIdx.x / p.G, c = blockIdx.x % p.G, chunk = blockIdx.y, r0 = blockIdx.z * 16;
  const int row = p.row_list ? p.row_list[ri] : ri;
  const int R = p.H / p.G, Rb = min(16, R - r0), h0 = c * R + r0;
  T* out = reinterpret_cast<T*>(p.out) + (size_t)row * p.ldo;
  if (p.slots[row] < 0) {  // inert row of a padded step
    if (chunk == 0)
      for (int i = threadIdx.x; i < Rb * p.dv; i += 256) stv(out + (size_t)h0 * p.dv + i, 0.f);
    return;
  }
  const int pos = p.positions[row], seq = p.seq_ids[row];
  const Vis v = vis_tiles(pos, pos, p.window, p.keep);
  if (chunk * kChunkTiles >= v.n) return;
  const int nact = (v.n + kChunkTiles - 1) / kChunkTiles;
  const int nt = min(kChunkTiles, v.n - chunk * kChunkTiles), nkey = nt * kTile;
  T* pf = reinterpret_cast<T*>(smem);                                   // mixed weights, B-operand order
  float* wt = reinterpret_cast<float*>(smem + kChunk * 16 * sizeof(T));  // [H][128]
  float* hm = wt + p.H * kChunk;                                        // [H] max
  float* hl = hm + p.H;                                                 // [H] 1 / sum
  const int g0 = p.talk ? 0 : h0, g1 = p.talk ? p.H : h0 + Rb;          // heads whose weights are needed
  // ---- statistics of every needed head: 16 lanes per head
  for (int h = g0 + (threadIdx.x >> 4); h < g1; h += 16) {
    const float* st = p.stat + ((size_t)ri * p.H + h) * p.nch * 2;
    float m = -INFINITY;
    for (int k = threadIdx.x & 15; k < nact; k += 16) m = fmaxf(m, st[2 * k]);
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) m = fmaxf(m, __shfl_xor(m, o, 64));
    float s = 0.f;
    for (int k = threadIdx.x & 15; k < nact; k += 16) s += st[2 * k + 1] > 0.f ? st[2 * k + 1] * __expf(st[2 * k] - m) : 0.f;
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
    if ((threadIdx.x & 15) == 0) {
      hm[h] = m;
      hl[h] = 1.f / s;
    }
  }
  __syncthreads();
  // ---- normalised weights of the chunk's keys (0 past the last tile)
  {
    const int j = threadIdx.x & (kChunk - 1);
    for (int h = g0 + (threadIdx.x >> 7); h < g1; h += 2) {
      float x = 0.f;
      if (j < nkey) {
        const float s = p.s[((size_t)ri * p.H + h) * p.nch * kChunk + chunk * kChunk + j];
        x = s == -INFINITY ? 0.f : __expf(s - hm[h]) * hl[h];
      }
      wt[h * kChunk + j] = x;
    }
  }
  __syncthreads();
  // ---- mixed weights of this kv head's query heads
  {
    const int j = threadIdx.x & (kChunk - 1);
    const int idx = ((j / M::KS) * 64 + 16 * ((j % M::KS) / M::EPL)) * M::EPL + j % M::EPL;
    for (int r = threadIdx.x >> 7; r < Rb; r += 2) {
      float x = 0.f;
      if (p.talk) {
        const float* tk = p.talk + (size_t)(h0 + r) * p.H;
        for (int g = 0; g < p.H; ++g) x += tk[g] * wt[g * kChunk + j];
      } else {
        x = wt[(h0 + r) * kChunk + j];
      }
      stv(pf + idx + r * M::EPL, x);
    }
  }
  __syncthreads();
  // ---- O^T = V^T . P^T: wave w takes 16-column tiles w, w + 4, ... of the values
  const int lane = lane_id(), w = threadIdx.x >> 6, rl = lane & 15, b = lane >> 4;
  constexpr int TPS = M::KS / kTile;                 // tiles per step (bf16 2, f32 1)
  constexpr int NST = kChunkTiles / TPS;
  const T* vb[NST];
  bool vok[NST];
#pragma unroll
  for (int s = 0; s < NST; ++s) {
    const int t = chunk * kChunkTiles + s * TPS + (TPS == 2 ? b >> 1 : 0);
    vok[s] = t < v.n;
    const int key = tile_of(v, vok[s] ? t : v.n - 1) * kTile;
    const int64_t blk = p.block_table[(int64_t)seq * p.table_stride + key / p.block_size];
    vb[s] = reinterpret_cast<const T*>(p.v) + blk * p.v_sb + (int64_t)c * p.v_sh + (int64_t)rl * p.block_size +
            key % p.block_size + (TPS == 2 ? (b & 1) : b) * M::EPL;
  }
  const int nz = gridDim.z;
  float* prow = p.part + ((size_t)ri * p.nch) * p.H * p.dv;
  const __amdgpu_buffer_rsrc_t rp = rsrc_f32(prow, (int64_t)p.nch * p.H * p.dv);
  for (int d = w * 16; d < p.dv; d += 64) {
    uint4 va[NST];
#pragma unroll
    for (int s = 0; s < NST; ++s)
      va[s] = vok[s] ? *reinterpret_cast<const uint4*>(vb[s] + (int64_t)d * p.block_size) : make_uint4(0, 0, 0, 0);
    f32x4 acc = {};
#pragma unroll
    for (int s = 0; s < NST; ++s)
      acc = M::mma(va[s], *reinterpret_cast<const uint4*>(pf + ((size_t)s * 64 + lane) * M::EPL), acc);
    if (rl >= Rb) continue;
    const int h = h0 + rl;
    if (nact == 1) {
      const float g = head_gate<T>(p, row, h);
#pragma unroll
      for (int i = 0; i < 4; ++i) stv(out + (size_t)h * p.dv + d + 4 * b + i, acc[i] * g);
    } else {
      const int64_t o = ((int64_t)chunk * p.H + h) * p.dv + d + 4 * b;
      st_sc1_f2(rp, o, acc[0], acc[1]);
      st_sc1_f2(rp, o + 2, acc[2], acc[3]);
    }
  }
  if (nact == 1) return;
  // ---- ticket; the last arriver adds the chunks in order
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (threadIdx.x == 0) {
    int* cnt = p.counters + ((size_t)ri * p.G + c) * nz + blockIdx.z;
    const int ticket = __hip_atomic_fetch_add(cnt, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    const int last = ticket == nact - 1;
    if (last) __hip_atomic_store(cnt, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    s_last = last;
  }
  __syncthreads();
  if (!s_last) return;
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
  for (int i = threadIdx.x * 2; i < Rb * p.dv; i += 512) {
    const int64_t o = (int64_t)h0 * p.dv + i;
    float a0 = 0.f, a1 = 0.f;
#pragma unroll 8
    for (int k = 0; k < nact; ++k) {
      const float2 x = ld_sc1_f2(rp, (int64_t)k * p.H * p.dv + o);
      a0 += x.x;
      a1 += x.y;
    }
    const float g = head_gate<T>(p, row, h0 + i / p.dv);
    stv(out + o, a0 * g);
    stv(out + o + 1, a1 * g);
  }
}

// ------------------------------------------------------------------------------------------ prefill form
constexpr int kTab = 1024;                  // block-table entries kept in LDS
constexpr int kNone = -1;

VWA_DEVICE void st_sc1_x4(__amdgpu_buffer_rsrc_t r, int off, const f32x4& v) {
  __builtin_amdgcn_raw_buffer_store_b128(__builtin_bit_cast(u32x4, v), r, off, 0, 16);
}
VWA_DEVICE f32x4 ld_sc1_x4(__amdgpu_buffer_rsrc_t r, int off) {
  return __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(r, off, 0, 16));
}

// every key of the tile visible to every query p0 .. p1 (no per-key masks needed)
VWA_DEVICE bool all_visible(int p0, int p1, int key0, int window, int keep) {
  return key0 + kTile - 1 <= p0 && (window <= 0 || p1 - key0 < window || key0 + kTile - 1 < keep);
}

// Pass 1: log2-sum-exp of every (query, head): a workgroup per (16 queries, kv head, RB query heads),
// the query fragments in registers, its 4 waves taking every fourth key tile (next tile's keys in
// flight).  lse[row][H] = max + log2(sum) of the scaled scores in log2 units.
template <int RB, int KSN>
__global__ __launch_bounds__(256) void talk_lse_kernel(TalkPrefillParams pp) {
  const TalkAttnParams& p = pp.a;
  __shared__ float red[4][RB][16][2];
  const int lane = lane_id(), w = threadIdx.x >> 6, rl = lane & 15, b = lane >> 4;
  const int lt = xcd_remap((int)blockIdx.x, pp.n_tiles * p.G);  // (a kv head's tiles share an XCD's L2)
  const int c = lt / pp.n_tiles, tile = lt % pp.n_tiles;
  const int row0 = pp.tiles[2 * tile], nq = pp.tiles[2 * tile + 1];
  const int R = p.H / p.G, r0 = blockIdx.y * RB, nr = min(RB, R - r0), nst = p.dk >> 5;
  const int pos0 = p.positions[row0], pos1 = pos0 + nq - 1, seq = p.seq_ids[row0];
  const int qrow = row0 + min(rl, nq - 1), qpos = pos0 + min(rl, nq - 1);
  const Vis v = vis_tiles(pos0, pos1, p.window, p.keep);
  const float sl2 = p.scale * kLog2e;
  const int* gtab = p.block_table + (int64_t)seq * p.table_stride;
  uint4 qf[RB][KSN];
#pragma unroll
  for (int r = 0; r < RB; ++r)
#pragma unroll
    for (int s = 0; s < KSN; ++s)
      if (s < nst)
        qf[r][s] = ld128(reinterpret_cast<const u16*>(p.q) + (size_t)qrow * p.ldq + (size_t)(c * R + r0 + min(r, nr - 1)) * p.dk +
                         b * 8 + s * 32);
  auto load_k = [&](uint4 (&kf)[KSN], int t) {
    const int key0 = tile_of(v, t) * kTile;
    const u16* kp = reinterpret_cast<const u16*>(p.k) + (int64_t)gtab[key0 / p.block_size] * p.k_sb + (int64_t)c * p.k_sh +
                    (int64_t)(key0 % p.block_size + rl) * p.dk + b * 8;
#pragma unroll
    for (int s = 0; s < KSN; ++s)
      if (s < nst) kf[s] = ld128(kp + s * 32);
  };
  float m[RB], l[RB];
#pragma unroll
  for (int r = 0; r < RB; ++r) {
    m[r] = -1e30f;
    l[r] = 0.f;
  }
  auto add_tile = [&](const uint4 (&kf)[KSN], int t) {
    const int key0 = tile_of(v, t) * kTile;
    const bool full = all_visible(pos0, pos1, key0, p.window, p.keep);
    bool vis[4] = {true, true, true, true};
    if (!full) {
#pragma unroll
      for (int i = 0; i < 4; ++i) vis[i] = sees(qpos, key0 + 4 * b + i, p.window, p.keep);
    }
#pragma unroll
    for (int r = 0; r < RB; ++r) {
      f32x4 a = {};
#pragma unroll
      for (int s = 0; s < KSN; ++s)
        if (s < nst) a = mfma16(as_bf16x8(kf[s]), as_bf16x8(qf[r][s]), a);
      float s[4], mn = m[r];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[i] = vis[i] ? a[i] * sl2 : -1e30f;
        mn = fmaxf(mn, s[i]);
      }
      float x = l[r] * __builtin_amdgcn_exp2f(m[r] - mn);
#pragma unroll
      for (int i = 0; i < 4; ++i) x += vis[i] ? __builtin_amdgcn_exp2f(s[i] - mn) : 0.f;
      l[r] = x;
      m[r] = mn;
    }
  };
  uint4 ka[KSN], kb[KSN];
  if (w < v.n) load_k(ka, w);
  for (int t = w; t < v.n; t += 8) {
    if (t + 4 < v.n) load_k(kb, t + 4);
    add_tile(ka, t);
    if (t + 4 >= v.n) break;
    if (t + 8 < v.n) load_k(ka, t + 8);
    add_tile(kb, t + 4);
  }
#pragma unroll
  for (int r = 0; r < RB; ++r) {
#pragma unroll
    for (int o = 16; o < 64; o <<= 1) {
      const float mo = __shfl_xor(m[r], o, 64), lo = __shfl_xor(l[r], o, 64), mn = fmaxf(m[r], mo);
      l[r] = l[r] * __builtin_amdgcn_exp2f(m[r] - mn) + lo * __builtin_amdgcn_exp2f(mo - mn);
      m[r] = mn;
    }
    if (b == 0) {
      red[w][r][rl][0] = m[r];
      red[w][r][rl][1] = l[r];
    }
  }
  __syncthreads();
  const int r = threadIdx.x >> 4, q = threadIdx.x & 15;
  if (r >= nr || q >= nq) return;
  float mm = -1e30f, ll = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) mm = fmaxf(mm, red[i][r][q][0]);
#pragma unroll
  for (int i = 0; i < 4; ++i) ll += red[i][r][q][1] * __builtin_amdgcn_exp2f(red[i][r][q][0] - mm);
  pp.lse[(size_t)(row0 + q) * p.H + c * R + r0 + r] = mm + __log2f(ll);
}

// rows [0 1 2 3] of 16 lanes of four registers, transposed: out_b row b' = in_b' row b
VWA_DEVICE void transpose4(unsigned& a, unsigned& b, unsigned& c, unsigned& d) {
  const auto r = __builtin_amdgcn_permlane32_swap(a, c, false, false);
  const auto s = __builtin_amdgcn_permlane32_swap(b, d, false, false);
  const auto x = __builtin_amdgcn_permlane16_swap(r[0], s[0], false, false);
  const auto y = __builtin_amdgcn_permlane16_swap(r[1], s[1], false, false);
  a = x[0];
  b = x[1];
  c = y[0];
  d = y[1];
}

// Pass 2.  GP, RP: kv heads and query heads per kv head in the padded head order h = c * RP + r; NV: (kv
// head, 16 value columns) tiles per wave; NW waves; KSN: 32-wide steps over the q / k dimensions.
// Heads are mixed on the MFMA: a weight x = hi + lo (two bf16, 16 mantissa bits) is one B operand with
// k = (hi | lo, head) against the talk matrix (bf16 as stored) repeated for both halves; the lanes hold
// every head of their own (query, key), so the operand is a 4 x 4 transpose of 16-lane groups.
// A tile's key rows enter the score product in the order 4 i + b (row 4 b + i), so the four results of one
// key element i are four consecutive keys.
// The tile's keys may be split over workgroups (blockIdx.y): their sums are added in order by the last
// one to finish.
template <int GP, int RP, int NV, int NW, int KSN>
struct PrefillCfg {
  static constexpr int HT = GP * RP, KEYS = NW * kTile, KG = KEYS / 32;
  static constexpr int MT = HT > 16 ? 2 : 1;                         // 16-row tiles of the mixed heads
  static constexpr int KM = HT > 16 ? 2 : 1;                         // 32-deep steps of the mixing
  static constexpr int P_BYTES = HT * KEYS * 16 * 2;                 // mixed weights
  static constexpr bool QL = HT * KSN <= 64;                         // query fragments in LDS (else L1 / L2)
  static size_t lds(int dk) { return P_BYTES + HT * 16 * 4 + kTab * 4 + (QL ? (size_t)HT * dk * 16 * 2 : 0); }
};

template <int GP, int RP, int NV, int NW, int KSN>
__global__ __launch_bounds__(NW * 64) void talk_prefill_kernel(TalkPrefillParams pp) {
  using C = PrefillCfg<GP, RP, NV, NW, KSN>;
  constexpr int HT = C::HT, KG = C::KG, HX = HT < 4 ? 4 : HT;
  constexpr int HS = KG * 4 * 16 * 16;                               // bytes of a head's mixed weights
  const TalkAttnParams& p = pp.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ int s_last;
  char* pm = smem;                                                   // [HT][KG][4][16 q][8 keys]
  float* lse = reinterpret_cast<float*>(smem + C::P_BYTES);          // [HT][16]
  int* btab = reinterpret_cast<int*>(lse + HT * 16);
  uint4* qs = reinterpret_cast<uint4*>(btab + kTab);                 // [HT][dk / 32][64]
  const int lane = lane_id(), w = threadIdx.x >> 6, rl = lane & 15, b = lane >> 4;
  const int bt = xcd_remap((int)blockIdx.x, pp.n_tiles);
  const int row0 = pp.tiles[2 * bt], nq = pp.tiles[2 * bt + 1];
  const int R = p.H / p.G, nst = p.dk >> 5;
  const int pos0 = p.positions[row0], pos1 = pos0 + nq - 1, seq = p.seq_ids[row0];
  const int qrow = row0 + min(rl, nq - 1), qpos = pos0 + min(rl, nq - 1);
  const Vis v = vis_tiles(pos0, pos1, p.window, p.keep);
  const int nit = (v.n + NW - 1) / NW, per = (nit + pp.splits - 1) / pp.splits;
  const int nact = (nit + per - 1) / per;                            // splits with work
  const int split = blockIdx.y;
  if (split >= nact) return;
  const int it0 = split * per, it1 = min(nit, it0 + per);
  const float sl2 = p.scale * kLog2e;
  const int* gtab = p.block_table + (int64_t)seq * p.table_stride;
  const int nblk = pos1 / p.block_size + 1;
  const bool tab = nblk <= kTab;
  if (tab)
    for (int i = threadIdx.x; i < nblk; i += NW * 64) btab[i] = gtab[i];
  for (int u = threadIdx.x; u < p.H * 16; u += NW * 64) {
    const int h = u >> 4, q = u & 15;
    lse[((h / R) * RP + h % R) * 16 + q] = pp.lse[(size_t)(row0 + min(q, nq - 1)) * p.H + h];
  }
  const u16* qp = reinterpret_cast<const u16*>(p.q) + (size_t)qrow * p.ldq + b * 8;
  if constexpr (C::QL) {
    for (int u = w; u < p.H * nst; u += NW) {
      const int h = u / nst, s = u % nst;
      qs[((size_t)((h / R) * RP + h % R) * nst + s) * 64 + lane] = ld128(qp + (size_t)h * p.dk + s * 32);
    }
  }
  uint4 tf[C::MT];                                                   // talk, A operand (both mixing steps use it)
#pragma unroll
  for (int mt = 0; mt < C::MT; ++mt) tf[mt] = reinterpret_cast<const uint4*>(pp.talk_frag)[mt * 64 + lane];
  __syncthreads();
  auto blk_of = [&](int key) -> int64_t {
    const int i = key / p.block_size;
    return tab ? btab[i] : gtab[i];
  };
  auto load_k = [&](uint4 (&kf)[KSN], int c, int t) {
    const int key0 = tile_of(v, t) * kTile;
    const u16* kp = reinterpret_cast<const u16*>(p.k) + blk_of(key0) * p.k_sb + (int64_t)c * p.k_sh +
                    (int64_t)(key0 % p.block_size + 4 * (rl & 3) + (rl >> 2)) * p.dk + b * 8;
#pragma unroll
    for (int s = 0; s < KSN; ++s)
      if (s < nst) kf[s] = ld128(kp + s * 32);
  };
  const int ndv = p.dv >> 4, nvt = p.G * ndv, nvw = (nvt + NW - 1) / NW, v0 = w * nvw;
  // value tiles of a wave in chunks of NC; a step is one chunk of one 32-key group
  constexpr int NC = NV < 4 ? NV : 4, CH = NV / NC, STEPS = KG * CH;
  static_assert(NV % NC == 0, "whole chunks");
  auto load_v = [&](uint4 (&vf)[NC], int it, int step) {
    const int key = tile_of(v, min(it * NW + 2 * (step / CH) + (b >> 1), v.n - 1)) * kTile;
    const u16* vp = reinterpret_cast<const u16*>(p.v) + blk_of(key) * p.v_sb + (int64_t)rl * p.block_size +
                    key % p.block_size + (b & 1) * 8;
#pragma unroll
    for (int n = 0; n < NC; ++n) {
      const int idx = min(v0 + min((step % CH) * NC + n, nvw - 1), nvt - 1);
      vf[n] = ld128(vp + (int64_t)(idx / ndv) * p.v_sh + (int64_t)(idx % ndv) * 16 * p.block_size);
    }
  };

  f32x4 acc[NV][RP] = {};
  uint4 kf[2][KSN];
  if (it0 * NW + w < v.n) load_k(kf[0], 0, it0 * NW + w);
  for (int it = it0; it < it1; ++it) {
    const int t = it * NW + w;
    char* pw = pm + (((w >> 1) * 4 + 2 * (w & 1)) * 16 + rl) * 16;   // [head][..][key chunk][q]
    uint4 vf[2][NC];
    if (t < v.n) {
      const int key0 = tile_of(v, t) * kTile;
      const bool full = all_visible(pos0, pos1, key0, p.window, p.keep);
      bool vis[4] = {true, true, true, true};
      if (!full) {
#pragma unroll
        for (int i = 0; i < 4; ++i) vis[i] = sees(qpos, key0 + 4 * i + b, p.window, p.keep);
      }
      // hi / lo parts of the weights, [key i][heads pairwise]
      unsigned xh[4][HX / 2], xl[4][HX / 2];
      float px[4] = {0.f, 0.f, 0.f, 0.f};  // the even head of a pair
#pragma unroll
      for (int c = 0; c < GP; ++c) {
        if (c + 1 < GP && c + 1 < p.G) load_k(kf[(c + 1) & 1], c + 1, t);
#pragma unroll
        for (int r = 0; r < RP; ++r) {
          const int h = c * RP + r;
          f32x4 a = {};
          const bool real = c < p.G && r < R;
          if (real) {
#pragma unroll
            for (int s = 0; s < KSN; ++s)
              if (s < nst) {
                uint4 qf;
                if constexpr (C::QL) qf = qs[((size_t)h * nst + s) * 64 + lane];
                else qf = ld128(qp + (size_t)(c * R + r) * p.dk + s * 32);
                a = mfma16(as_bf16x8(kf[c & 1][s]), as_bf16x8(qf), a);
              }
          }
          const float ls = lse[h * 16 + rl];
          float x[4];
#pragma unroll
          for (int i = 0; i < 4; ++i) x[i] = real && vis[i] ? __builtin_amdgcn_exp2f(a[i] * sl2 - ls) : 0.f;
          if (HT == 1 || (h & 1)) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const float e = HT == 1 ? x[i] : px[i], o = HT == 1 ? 0.f : x[i];
              const unsigned hi = pack2(e, o);
              xh[i][h >> 1] = hi;
              xl[i][h >> 1] = pack2(e - __uint_as_float(hi << 16), o - __uint_as_float(hi & 0xffff0000u));
            }
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i) px[i] = x[i];
          }
          // (bounds how far ahead the query fragments are read: unbounded, their registers spill)
          if ((r & 1) == 1 || RP == 1) __builtin_amdgcn_sched_barrier(0);
        }
      }
      if constexpr (HT < 4) {
#pragma unroll
        for (int i = 0; i < 4; ++i) xh[i][1] = xl[i][1] = 0u;
      }
      // next iteration's first keys, this one's first values
      if (t + NW < v.n && it + 1 < it1) load_k(kf[0], 0, t + NW);
      load_v(vf[0], it, 0);
      // per key element: B operands by transposing the lane groups' blocks of 8 heads (4 registers), the
      // mixed weights of keys 4 i .. 4 i + 3 of every head, and their bf16 quads to LDS
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        uint4 bm[C::KM][4];  // [mixing step][source lane group]
#pragma unroll
        for (int ks = 0; ks < C::KM; ++ks) {
          unsigned o[4][4];  // [source group][register]
#pragma unroll
          for (int g = 0; g < 4; ++g) {
            unsigned q0, q1, q2, q3;
            if constexpr (HT == 32) {
              const unsigned (&x)[HX / 2] = ks ? xl[i] : xh[i];
              q0 = x[g], q1 = x[4 + g], q2 = x[8 + g], q3 = x[12 + g];
            } else if constexpr (HT == 16) {
              q0 = xh[i][g], q1 = xh[i][4 + g], q2 = xl[i][g], q3 = xl[i][4 + g];
            } else if constexpr (HT == 8) {
              q0 = xh[i][g], q1 = xl[i][g], q2 = 0u, q3 = 0u;
            } else {
              q0 = g < 2 ? xh[i][g & 1] : xl[i][g & 1], q1 = 0u, q2 = 0u, q3 = 0u;
            }
            transpose4(q0, q1, q2, q3);
            o[0][g] = q0, o[1][g] = q1, o[2][g] = q2, o[3][g] = q3;
          }
#pragma unroll
          for (int g = 0; g < 4; ++g) bm[ks][g] = make_uint4(o[g][0], o[g][1], o[g][2], o[g][3]);
        }
#pragma unroll
        for (int mt = 0; mt < C::MT; ++mt) {
          f32x4 y[4];
#pragma unroll
          for (int g = 0; g < 4; ++g) {
            f32x4 a = {};
#pragma unroll
            for (int ks = 0; ks < C::KM; ++ks) a = mfma16(as_bf16x8(tf[mt]), as_bf16x8(bm[ks][g]), a);
            y[g] = a;
          }
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int h = 16 * mt + 4 * b + e;
            if (HT >= 16 || h < HT)
              *reinterpret_cast<uint2*>(pw + h * HS + (i >> 1) * 256 + (i & 1) * 8) =
                  make_uint2(pack2(y[0][e], y[1][e]), pack2(y[2][e], y[3][e]));
          }
        }
      }
    } else {
      load_v(vf[0], it, 0);
#pragma unroll
      for (int mt = 0; mt < C::MT; ++mt)
#pragma unroll
        for (int ch = 0; ch < 2; ++ch)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int h = 16 * mt + 4 * b + i;
            if (HT >= 16 || h < HT) *reinterpret_cast<uint4*>(pw + h * HS + ch * 256) = make_uint4(0, 0, 0, 0);
          }
    }
    lds_sync();
    uint4 pf[RP];
#pragma unroll
    for (int st = 0; st < STEPS; ++st) {
      const int kg = st / CH;
      if (it * NW + 2 * kg >= v.n) break;
      if (st + 1 < STEPS && it * NW + 2 * ((st + 1) / CH) < v.n) load_v(vf[(st + 1) & 1], it, st + 1);
#pragma unroll
      for (int n = 0; n < NC; ++n) {
        const int u = (st % CH) * NC + n, idx = v0 + u;
        if (u >= nvw || idx >= nvt) break;
        const int c = idx / ndv;
        if (u == 0 || c != (idx - 1) / ndv) {  // (the kv head's mixed weights serve all of its value tiles)
#pragma unroll
          for (int r = 0; r < RP; ++r)
            if (r < R) pf[r] = *reinterpret_cast<const uint4*>(pm + (c * RP + r) * HS + ((kg * 4 + b) * 16 + rl) * 16);
        }
#pragma unroll
        for (int r = 0; r < RP; ++r)
          if (r < R) acc[u][r] = mfma16(as_bf16x8(vf[st & 1][n]), as_bf16x8(pf[r]), acc[u][r]);
      }
    }
    lds_sync();
  }
  if (nact > 1) {
    // ---- every split's sums out (sc1), a ticket, and the last one adds them in order
    constexpr int kWave = NV * RP * 64 * 16, kPart = NW * kWave;     // bytes per wave / workgroup
    float* base = pp.part + (size_t)bt * pp.splits * (kPart / 4);
    const __amdgpu_buffer_rsrc_t rp = rsrc_f32(base, (int64_t)pp.splits * (kPart / 4));
    const int at = w * kWave + lane * 16;
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int r = 0; r < RP; ++r) st_sc1_x4(rp, split * kPart + at + (n * RP + r) * 1024, acc[n][r]);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (threadIdx.x == 0) {
      const int ticket = __hip_atomic_fetch_add(pp.tickets + bt, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      const int last = ticket == nact - 1;
      if (last) __hip_atomic_store(pp.tickets + bt, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      s_last = last;
    }
    __syncthreads();
    if (!s_last) return;
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int r = 0; r < RP; ++r) acc[n][r] = ld_sc1_x4(rp, at + (n * RP + r) * 1024);
    for (int s = 1; s < nact; ++s)
#pragma unroll
      for (int n = 0; n < NV; ++n)
#pragma unroll
        for (int r = 0; r < RP; ++r) acc[n][r] += ld_sc1_x4(rp, s * kPart + at + (n * RP + r) * 1024);
  }
  // ---- gate, scale, store: lane (query rl, value columns 4b .. 4b+3 of the tile)
  if (rl >= nq) return;
#pragma unroll
  for (int n = 0; n < NV; ++n) {
    const int idx = v0 + n;
    if (n >= nvw || idx >= nvt) break;
    const int c = idx / ndv, d = (idx % ndv) * 16 + 4 * b;
#pragma unroll
    for (int r = 0; r < RP; ++r) {
      if (r >= R) break;
      const int h = c * R + r;
      const float g = head_gate<u16>(p, qrow, h);
      uint2 o;
      o.x = pack2(acc[n][r][0] * g, acc[n][r][1] * g);
      o.y = pack2(acc[n][r][2] * g, acc[n][r][3] * g);
      *reinterpret_cast<uint2*>(reinterpret_cast<u16*>(p.out) + (size_t)qrow * p.ldo + (size_t)h * p.dv + d) = o;
    }
  }
}

int pow2_up(int n) {
  int p = 1;
  while (p < n) p <<= 1;
  return p;
}

constexpr size_t kMaxLds = 160 * 1024;

// what a call wants: only whether the sizes have an instantiation, its partial floats per tile and split,
// or the launch
enum Want { WANT_FIT, WANT_PART, WANT_LAUNCH };

template <int GP, int RP, int NV, int NW, int KSN>
int64_t prefill_cfg(const TalkPrefillParams& p, hipStream_t st, Want want) {
  using C = PrefillCfg<GP, RP, NV, NW, KSN>;
  if (C::lds(p.a.dk) > kMaxLds - 64) return -10;
  if (want == WANT_FIT) return 0;
  if (want == WANT_PART) return (int64_t)NW * NV * RP * 256;
  const int R = p.a.H / p.a.G;
  constexpr int RB = RP < 4 ? RP : 4;
  hipLaunchKernelGGL((talk_lse_kernel<RB, KSN>), dim3(p.n_tiles * p.a.G, (R + RB - 1) / RB), dim3(256), 0, st, p);
  hipLaunchKernelGGL((talk_prefill_kernel<GP, RP, NV, NW, KSN>), dim3(p.n_tiles, p.splits), dim3(NW * 64),
                     (C::lds(p.a.dk)), st, p);
  return 0;
}

template <int GP, int RP>
int64_t prefill_sizes(const TalkPrefillParams& p, hipStream_t st, Want want) {
  constexpr int HT = GP * RP;
  constexpr int NW = HT > 16 ? 4 : 8;       // 32 heads: 4 waves with twice the registers
  constexpr int N1 = (GP * 8 + NW - 1) / NW, N2 = (GP * 16 + NW - 1) / NW;   // dv <= 128 / <= 256
  const int need = (p.a.G * (p.a.dv >> 4) + NW - 1) / NW;
  if (need <= N1) {
    if (p.a.dk <= 128) return prefill_cfg<GP, RP, N1, NW, 4>(p, st, want);
    return prefill_cfg<GP, RP, N1, NW, 8>(p, st, want);
  }
  if constexpr (HT <= 16) {
    if (need <= N2) {
      if (p.a.dk <= 128) return prefill_cfg<GP, RP, N2, NW, 4>(p, st, want);
      return prefill_cfg<GP, RP, N2, NW, 8>(p, st, want);
    }
  }
  return -10;
}

int64_t dispatch_prefill(const TalkPrefillParams& p, hipStream_t st, Want want) {
  const TalkAttnParams& a = p.a;
  if (a.H < 1 || a.G < 1 || a.H % a.G || a.dk % 32 || a.dk > 256 || a.dv % 16 || a.dv < 16) return -10;
  switch (pow2_up(a.G) * 100 + pow2_up(a.H / a.G)) {
    case 101: return prefill_sizes<1, 1>(p, st, want);
    case 102: return prefill_sizes<1, 2>(p, st, want);
    case 104: return prefill_sizes<1, 4>(p, st, want);
    case 108: return prefill_sizes<1, 8>(p, st, want);
    case 201: return prefill_sizes<2, 1>(p, st, want);
    case 202: return prefill_sizes<2, 2>(p, st, want);
    case 204: return prefill_sizes<2, 4>(p, st, want);
    case 208: return prefill_sizes<2, 8>(p, st, want);
    case 401: return prefill_sizes<4, 1>(p, st, want);
    case 402: return prefill_sizes<4, 2>(p, st, want);
    case 404: return prefill_sizes<4, 4>(p, st, want);
    case 408: return prefill_sizes<4, 8>(p, st, want);
    case 801: return prefill_sizes<8, 1>(p, st, want);
    case 802: return prefill_sizes<8, 2>(p, st, want);
    case 804: return prefill_sizes<8, 4>(p, st, want);
    case 1601: return prefill_sizes<16, 1>(p, st, want);
    case 1602: return prefill_sizes<16, 2>(p, st, want);
    default: return -10;
  }
}

int check_attn(const TalkAttnParams& p) {
  if (p.rows < 1 || p.G < 1 || p.H < 1 || p.H % p.G || p.block_size % kTile || p.dk % 32 || p.dv % 16) return -1;
  if (p.window < 0 || p.keep < 0) return -2;
  if ((p.k_sh | p.k_sb | p.v_sh | p.v_sb | p.ldq) % 8) return -3;
  return 0;
}

}  // namespace

extern "C" int vwa_talk_attention(const TalkAttnParams* p, hipStream_t st) {
  const int rc = check_attn(*p);
  if (rc) return rc;
  if (p->nch < 1 || !p->s || !p->stat || !p->part || !p->counters) return -4;
  const size_t lds = p->f32 ? mix_lds<float>(p->H) : mix_lds<u16>(p->H);
  if (lds > kMaxLds - 64 || (int64_t)p->nch * p->H * p->dv * 4 >= (1ll << 31)) return -5;
  const dim3 grid(p->rows * p->G, p->nch, (p->H / p->G + 15) / 16), block(256);
  if (p->f32) {
    hipLaunchKernelGGL((talk_scores_kernel<float>), grid, block, 0, st, *p);
    hipLaunchKernelGGL((talk_mix_kernel<float>), grid, block, lds, st, *p);
  } else {
    hipLaunchKernelGGL((talk_scores_kernel<u16>), grid, block, 0, st, *p);
    hipLaunchKernelGGL((talk_mix_kernel<u16>), grid, block, lds, st, *p);
  }
  return (int)hipGetLastError();
}

extern "C" int64_t vwa_talk_prefill_part(int H, int G, int dk, int dv) {
  TalkPrefillParams p{};
  p.a.H = H;
  p.a.G = G;
  p.a.dk = dk;
  p.a.dv = dv;
  return dispatch_prefill(p, nullptr, WANT_PART);
}

extern "C" int vwa_talk_prefill(const TalkPrefillParams* p, hipStream_t st) {
  const int rc = check_attn(p->a);
  if (rc) return rc;
  if (p->a.f32 || p->n_tiles < 1 || !p->tiles || !p->talk_frag || !p->lse || p->splits < 1 || p->a.ldo % 4) return -6;
  if (p->splits > 1) {
    const int64_t part = dispatch_prefill(*p, st, WANT_PART);
    if (!p->part || !p->tickets || part < 0 || part * p->splits * 4 >= (1ll << 31)) return -7;
  }
  const int64_t r = dispatch_prefill(*p, st, WANT_LAUNCH);
  if (r) return (int)r;
  return (int)hipGetLastError();
}
