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
//     launch B recomputes them (a wave per few heads), mixes the heads on the MFMA and multiplies by V^T,
//     the weights passing between the waves through LDS in B-operand order.
#include "common.h"
#include "mq_attention.h"
#include "stack_kernels.h"
#include "stack_types.h"

using namespace vwa;

namespace {

constexpr int kTile = 16;                  // keys per tile
constexpr float kLog2e = 1.4426950408889634f;

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

VWA_DEVICE void st_sc1_x4(__amdgpu_buffer_rsrc_t r, int off, const f32x4& v) {
  __builtin_amdgcn_raw_buffer_store_b128(__builtin_bit_cast(u32x4, v), r, off, 0, 16);
}
VWA_DEVICE f32x4 ld_sc1_x4(__amdgpu_buffer_rsrc_t r, int off) {
  return __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(r, off, 0, 16));
}

// ------------------------------------------------------------------------------------------ rows form
constexpr int kChunkTiles = 8;             // most tiles of a workgroup's chunk
constexpr int kChunk = kTile * kChunkTiles;

// A row's visible tiles are dealt evenly to the fewest chunks; chunk c holds tiles c * per ..
struct Chunks {
  int per, n;
};
VWA_DEVICE Chunks chunks_of(int tiles) {
  const int k = (tiles + kChunkTiles - 1) / kChunkTiles, per = (tiles + k - 1) / k;
  return Chunks{per, (tiles + per - 1) / per};
}

template <class T>
__global__ __launch_bounds__(256) void talk_scores_kernel(TalkAttnParams p) {
  using M = MM<T>;
  constexpr int NU = kChunkTiles / 4;                // tiles per wave
  __shared__ float sm[4][16][2];
  const int ri = blockIdx.x / p.G, c = blockIdx.x % p.G, chunk = blockIdx.y, r0 = blockIdx.z * 16;
  const int row = p.row_list ? p.row_list[ri] : ri;
  if (p.slots[row] < 0) return;
  const int pos = p.positions[row], seq = p.seq_ids[row];
  const Vis v = vis_tiles(pos, pos, p.window, p.keep);
  const Chunks ck = chunks_of(v.n);
  if (chunk >= ck.n) return;
  const int R = p.H / p.G, Rb = min(16, R - r0);
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rl = lane & 15, b = lane >> 4;
  const T* q = reinterpret_cast<const T*>(p.q) + (size_t)row * p.ldq + (size_t)(c * R + r0 + min(rl, Rb - 1)) * p.dk + b * M::EPL;
  const int lb = __builtin_ctz(p.block_size);
  const T* kp[NU];
  int key0[NU];
  bool ok[NU];
#pragma unroll
  for (int u = 0; u < NU; ++u) {
    const int lt = w + 4 * u, t = chunk * ck.per + lt;
    ok[u] = lt < ck.per && t < v.n;
    key0[u] = tile_of(v, ok[u] ? t : v.n - 1) * kTile;
    const int64_t blk = p.block_table[(int64_t)seq * p.table_stride + (key0[u] >> lb)];
    kp[u] = reinterpret_cast<const T*>(p.k) + blk * p.k_sb + (int64_t)c * p.k_sh +
            (int64_t)((key0[u] & (p.block_size - 1)) + rl) * p.dk + b * M::EPL;
  }
  f32x4 acc[NU] = {};
#pragma unroll 4
  for (int k = 0; k < p.dk; k += M::KS) {
    const uint4 qf = *reinterpret_cast<const uint4*>(q + k);
#pragma unroll
    for (int u = 0; u < NU; ++u) acc[u] = M::mma(*reinterpret_cast<const uint4*>(kp[u] + k), qf, acc[u]);
  }
  // lane (column rl = head, keys 4b .. 4b+3 of both tiles): mask, store, chunk statistics
  float mx = -INFINITY;
#pragma unroll
  for (int u = 0; u < NU; ++u)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const bool vis = ok[u] && sees(pos, key0[u] + 4 * b + i, p.window, p.keep);
      acc[u][i] = vis ? acc[u][i] * p.scale : -INFINITY;
      mx = fmaxf(mx, acc[u][i]);
    }
  if (rl < Rb) {
#pragma unroll
    for (int u = 0; u < NU; ++u)
      if (ok[u])
        *reinterpret_cast<float4*>(p.s + ((size_t)ri * p.H + c * R + r0 + rl) * p.nch * kChunk +
                                   chunk * kChunk + (w + 4 * u) * kTile + 4 * b) =
            make_float4(acc[u][0], acc[u][1], acc[u][2], acc[u][3]);
  }
  mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
  mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
  float l = 0.f;
#pragma unroll
  for (int u = 0; u < NU; ++u)
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

// LDS: statistics [H][2], weights [H][keys] f32, mixed weights [keys / KS][64][16 B]
template <class T>
size_t mix_lds(int H) { return (size_t)H * (2 + kChunk) * 4 + kChunk * 16 * sizeof(T); }

template <class T>
__global__ __launch_bounds__(256) void talk_mix_kernel(TalkAttnParams p) {
  using M = MM<T>;
  constexpr int HP = 256 / kChunk;                   // heads side by side over the threads
  static_assert(HP == 2);
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
  const Chunks ck = chunks_of(v.n);
  if (chunk >= ck.n) return;
  const int nact = ck.n, t0 = chunk * ck.per, nt = min(ck.per, v.n - t0), nkey = nt * kTile;
  T* pf = reinterpret_cast<T*>(smem);                                   // mixed weights, B-operand order
  float* wt = reinterpret_cast<float*>(smem + kChunk * 16 * sizeof(T));  // [H][keys]
  float* hm = wt + p.H * kChunk;                                        // [H] max
  float* hl = hm + p.H;                                                 // [H] 1 / sum
  const int g0 = p.talk ? 0 : h0, g1 = p.talk ? p.H : h0 + Rb;          // heads whose weights are needed
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rl = lane & 15, b = lane >> 4;
  // ---- everything that is read is requested first: the scores of this thread's (key, heads), the first
  // value tiles of this wave (16-column tiles w, w + 4, ...), the chunk statistics
  constexpr int kPre = 16 / HP;
  const int j = threadIdx.x & (kChunk - 1), hp = w >> 1;                // key, first head
  const float* srow = p.s + (size_t)ri * p.H * p.nch * kChunk + chunk * kChunk + j;
  float sv[kPre];
#pragma unroll
  for (int k = 0; k < kPre; ++k) sv[k] = srow[(size_t)min(g0 + hp + HP * k, g1 - 1) * p.nch * kChunk];
  constexpr int TPS = M::KS / kTile;                 // tiles per step (bf16 2, f32 1)
  constexpr int NST = kChunkTiles / TPS;
  const int lb = __builtin_ctz(p.block_size);
  const T* vb[NST];
  bool vok[NST];
#pragma unroll
  for (int s = 0; s < NST; ++s) {
    const int lt = s * TPS + (TPS == 2 ? b >> 1 : 0);
    vok[s] = lt < nt;
    const int key = tile_of(v, vok[s] ? t0 + lt : v.n - 1) * kTile;
    const int64_t blk = p.block_table[(int64_t)seq * p.table_stride + (key >> lb)];
    vb[s] = reinterpret_cast<const T*>(p.v) + blk * p.v_sb + (int64_t)c * p.v_sh + (int64_t)rl * p.block_size +
            (key & (p.block_size - 1)) + (TPS == 2 ? (b & 1) : b) * M::EPL;
  }
  uint4 va[NST], vn[NST];
  auto load_v = [&](uint4 (&x)[NST], int d) {
#pragma unroll
    for (int s = 0; s < NST; ++s)
      x[s] = vok[s] ? *reinterpret_cast<const uint4*>(vb[s] + (int64_t)min(d, p.dv - 16) * p.block_size) : make_uint4(0, 0, 0, 0);
  };
  load_v(va, w * 16);
  load_v(vn, w * 16 + 64);
  // ---- statistics of every needed head: 16 lanes per head
  for (int h = g0 + (threadIdx.x >> 4); h < g1; h += 16) {
    const float* st = p.stat + ((size_t)ri * p.H + h) * p.nch * 2;
    float m = -INFINITY, s = 0.f;
    for (int k = threadIdx.x & 15; k < nact; k += 16) {
      const float2 ms = *reinterpret_cast<const float2*>(st + 2 * k);
      const float mn = fmaxf(m, ms.x);
      if (ms.y > 0.f) s = (s > 0.f ? s * __expf(m - mn) : 0.f) + ms.y * __expf(ms.x - mn);
      m = mn;
    }
#pragma unroll
    for (int o = 8; o > 0; o >>= 1) {
      const float mo = __shfl_xor(m, o, 64), so = __shfl_xor(s, o, 64), mn = fmaxf(m, mo);
      s = (s > 0.f ? s * __expf(m - mn) : 0.f) + (so > 0.f ? so * __expf(mo - mn) : 0.f);
      m = mn;
    }
    if ((threadIdx.x & 15) == 0) {
      hm[h] = m;
      hl[h] = 1.f / s;
    }
  }
  __syncthreads();
  // ---- normalised weights of the chunk's keys (0 past the last tile)
  auto weight = [&](int h, float s) { wt[h * kChunk + j] = j < nkey && s != -INFINITY ? __expf(s - hm[h]) * hl[h] : 0.f; };
#pragma unroll
  for (int k = 0; k < kPre; ++k)
    if (g0 + hp + HP * k < g1) weight(g0 + hp + HP * k, sv[k]);
  for (int h = g0 + hp + HP * kPre; h < g1; h += HP) weight(h, srow[(size_t)h * p.nch * kChunk]);
  __syncthreads();
  // ---- mixed weights of this kv head's query heads
  {
    const int idx = ((j / M::KS) * 64 + 16 * ((j % M::KS) / M::EPL)) * M::EPL + j % M::EPL;
    for (int r = hp; r < Rb; r += HP) {
      float x = 0.f;
      if (p.talk) {
        const float* tk = p.talk + (size_t)(h0 + r) * p.H;  // (uniform per wave: scalar loads)
#pragma unroll 8
        for (int g = 0; g < p.H; ++g) x += tk[g] * wt[g * kChunk + j];
      } else {
        x = wt[(h0 + r) * kChunk + j];
      }
      stv(pf + idx + r * M::EPL, x);
    }
  }
  __syncthreads();
  // ---- O^T = V^T . P^T
  const int nz = gridDim.z;
  float* prow = p.part + ((size_t)ri * p.nch) * p.H * p.dv;
  const __amdgpu_buffer_rsrc_t rp = rsrc_f32(prow, (int64_t)p.nch * p.H * p.dv);
  for (int d = w * 16; d < p.dv; d += 64) {
    f32x4 acc = {};
#pragma unroll
    for (int s = 0; s < NST; ++s)
      acc = M::mma(va[s], *reinterpret_cast<const uint4*>(pf + ((size_t)s * 64 + lane) * M::EPL), acc);
#pragma unroll
    for (int s = 0; s < NST; ++s) va[s] = vn[s];
    if (d + 128 < p.dv) load_v(vn, d + 128);
    if (rl >= Rb) continue;
    const int h = h0 + rl;
    if (nact == 1) {
      const float g = head_gate<T>(p, row, h);
#pragma unroll
      for (int i = 0; i < 4; ++i) stv(out + (size_t)h * p.dv + d + 4 * b + i, acc[i] * g);
    } else {
      st_sc1_x4(rp, (int)((((int64_t)chunk * p.H + h) * p.dv + d + 4 * b) * 4), acc);
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
constexpr int kTab = 1024;                  // tiles a query tile may see (their cache places are kept in LDS)

// cache place of every visible tile: block * (tiles per block) + tile in the block
VWA_DEVICE void tile_table(const TalkAttnParams& p, const Vis& v, int seq, int* tab, int threads) {
  const int* gtab = p.block_table + (int64_t)seq * p.table_stride;
  const int lb = __builtin_ctz(p.block_size) - 4;           // log2 of the tiles per block
  for (int t = threadIdx.x; t < v.n; t += threads) {
    const int tl = tile_of(v, t);
    tab[t] = (gtab[tl >> lb] << lb) + (tl & ((1 << lb) - 1));
  }
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
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rl = lane & 15, b = lane >> 4;
  const int lt = xcd_remap((int)blockIdx.x, pp.n_tiles * p.G);  // (a kv head's tiles share an XCD's L2)
  const int c = lt / pp.n_tiles, tile = lt % pp.n_tiles;
  const int row0 = pp.tiles[2 * tile], nq = pp.tiles[2 * tile + 1];
  const int R = p.H / p.G, r0 = blockIdx.y * RB, nr = min(RB, R - r0), nst = p.dk >> 5;
  const int pos0 = p.positions[row0], pos1 = pos0 + nq - 1, seq = p.seq_ids[row0];
  const int qrow = row0 + min(rl, nq - 1), qpos = pos0 + min(rl, nq - 1);
  const Vis v = vis_tiles(pos0, pos1, p.window, p.keep);
  const float sl2 = p.scale * kLog2e;
  __shared__ int tab[kTab];
  tile_table(p, v, seq, tab, 256);
  const int lb = __builtin_ctz(p.block_size) - 4;
  // (steps past dk: the query fragment is zero, the key fragment repeats the last step)
  uint4 qf[RB][KSN];
#pragma unroll
  for (int r = 0; r < RB; ++r)
#pragma unroll
    for (int s = 0; s < KSN; ++s) {
      qf[r][s] = ld128(reinterpret_cast<const u16*>(p.q) + (size_t)qrow * p.ldq + (size_t)(c * R + r0 + min(r, nr - 1)) * p.dk +
                       b * 8 + min(s, nst - 1) * 32);
      if (s >= nst) qf[r][s] = make_uint4(0, 0, 0, 0);
    }
  __syncthreads();
  const u16* kbase = reinterpret_cast<const u16*>(p.k) + (int64_t)c * p.k_sh + rl * p.dk + b * 8;
  auto load_k = [&](uint4 (&kf)[KSN], int t) {
    const int ts = __builtin_amdgcn_readfirstlane(tab[min(t, v.n - 1)]);
    const u16* kp = kbase + (int64_t)(ts >> lb) * p.k_sb + (ts & ((1 << lb) - 1)) * kTile * p.dk;
#pragma unroll
    for (int s = 0; s < KSN; ++s) kf[s] = ld128(kp + min(s, nst - 1) * 32);
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
      for (int s = 0; s < KSN; ++s) a = mfma16(as_bf16x8(kf[s]), as_bf16x8(qf[r][s]), a);
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
  load_k(ka, w);
  for (int t = w; t < v.n; t += 8) {
    load_k(kb, t + 4);
    add_tile(ka, t);
    if (t + 4 >= v.n) break;
    load_k(ka, t + 8);
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

// Pass 2.  GP, RP: kv heads and query heads per kv head in the padded head order h = c * RP + r; NV: (kv
// head, 16 value columns) tiles per wave; KSN: 32-wide steps over the q / k dimensions.  8 waves walk
// the keys 32 (few heads: 64) at a time, in three stages with two barriers:
//   scores   a wave owns HW heads (their query fragments stay in its registers) and two key tiles; the
//            normalised weights x go to LDS as hi + lo bf16 pairs (16 mantissa bits together), in the
//            B-operand order of the mixing: k = (hi | lo, head), column = query, one block per key
//   mixing   a wave takes 4 keys: talk (bf16 as stored, repeated for both halves) times that block on
//            the MFMA; the mixed weights go back to LDS as bf16 in the B-operand order of the values
//   values   a wave owns NV value tiles of a kv head's query heads: O^T += V^T . P^T
// The values stage of one round and the scores of the next lie between the same two barriers.
// The tile's keys may be split over workgroups (blockIdx.y): their sums are added in order by the last
// one to finish.
constexpr int kPW = 8;                                               // waves
template <int GP, int RP, int NV, int KSN>
struct PrefillCfg {
  static constexpr int HT = GP * RP, HX = HT < 4 ? 4 : HT;
  static constexpr int KT = HX == 4 ? 4 : 2, KEYS = KT * kTile, KG = KT / 2;   // tiles, keys, 32-key groups per round
  static constexpr int HW = HX > kPW ? HX / kPW : 1;                 // heads per wave
  static constexpr int HWAVES = HX / HW;                             // waves over the heads; the others take other tiles
  static constexpr int NCW = HW > RP ? HW / RP : 1;                  // kv heads per wave
  static constexpr int MT = HT > 16 ? 2 : 1;                         // 16-row tiles of the mixed heads
  static constexpr int KM = HT > 16 ? 2 : 1;                         // 32-deep steps of the mixing
  // next keys requested after the values (not before the mixing): their registers would not fit beside
  // the accumulators and query fragments
  static constexpr bool LATE_K = NV * RP * 4 + HW * KSN * 4 > 128;
  static constexpr int NC = LATE_K ? (NV < 2 ? NV : 2) : NV < 4 ? NV : 4;   // value tiles loaded ahead
  static constexpr int X_BYTES = KEYS * KM * 1024, P_BYTES = HX * KEYS * 16 * 2;
  static constexpr int LDS = X_BYTES + P_BYTES + 2 * HX * 16 * 4 + kTab * 4;
};

// ONE: every wave's value tiles belong to one kv head (its mixed weights are read once per 32 keys)
template <int GP, int RP, int NV, int KSN, bool ONE>
__global__ __launch_bounds__(kPW * 64) void talk_prefill_kernel(TalkPrefillParams pp) {
  using C = PrefillCfg<GP, RP, NV, KSN>;
  constexpr int HT = C::HT, HX = C::HX, HW = C::HW, KG = C::KG, KT = C::KT;
  constexpr int HS = KG * 4 * 16 * 16;                               // bytes of a head's mixed weights
  constexpr int KB = C::KM * 1024;                                   // bytes of a key's mixing operand
  const TalkAttnParams& p = pp.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ int s_last;
  char* xm = smem;                                                   // [KEYS][KM][64][16 B]
  char* pm = smem + C::X_BYTES;                                      // [HX][KG][4][16 q][8 keys]
  float* lse = reinterpret_cast<float*>(pm + C::P_BYTES);            // [HX][16]
  float* gate = lse + HX * 16;                                       // [HX][16] output factors
  int* btab = reinterpret_cast<int*>(gate + HX * 16);
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rl = lane & 15, b = lane >> 4;
  const int bt = xcd_remap((int)blockIdx.x, pp.n_tiles);
  const int row0 = pp.tiles[2 * bt], nq = pp.tiles[2 * bt + 1];
  const int R = p.H / p.G, nst = p.dk >> 5;
  const int pos0 = p.positions[row0], pos1 = pos0 + nq - 1, seq = p.seq_ids[row0];
  const int qrow = row0 + min(rl, nq - 1), qpos = pos0 + min(rl, nq - 1);
  const Vis v = vis_tiles(pos0, pos1, p.window, p.keep);
  const int nit = (v.n + KT - 1) / KT, per = (nit + pp.splits - 1) / pp.splits;
  const int nact = (nit + per - 1) / per;                            // splits with work
  const int split = blockIdx.y;
  if (split >= nact) return;
  const int it0 = split * per, it1 = min(nit, it0 + per);
  const float sl2 = p.scale * kLog2e;
  tile_table(p, v, seq, btab, kPW * 64);
  const int lb = __builtin_ctz(p.block_size) - 4, lm = (1 << lb) - 1;
  // (padding heads: weights exp2(-huge) = 0)
  for (int u = threadIdx.x; u < HX * 16; u += kPW * 64)
    if ((u >> 4) / RP >= p.G || (u >> 4) % RP >= R) lse[u] = 1e30f;
  for (int u = threadIdx.x; u < p.H * 16; u += kPW * 64) {
    const int h = u >> 4, q = u & 15;
    const int at = ((h / R) * RP + h % R) * 16 + q;
    lse[at] = pp.lse[(size_t)(row0 + min(q, nq - 1)) * p.H + h];
    gate[at] = head_gate<u16>(p, row0 + min(q, nq - 1), h);
  }
  // (operand slots no head writes -- padding heads, blocks past 2 HT -- stay zero)
  for (int u = threadIdx.x; u < C::X_BYTES / 16; u += kPW * 64) reinterpret_cast<uint4*>(xm)[u] = make_uint4(0, 0, 0, 0);
  // this wave's heads and tiles of a round
  const int hw0 = (w % C::HWAVES) * HW, tw0 = (w / C::HWAVES) * 2;
  const u16* qp = reinterpret_cast<const u16*>(p.q) + (size_t)qrow * p.ldq + b * 8;
  uint4 qf[HW][KSN];
  float ls[HW];
#pragma unroll
  for (int k = 0; k < HW; ++k) {
    const int c = min((hw0 + k) / RP, p.G - 1), r = min((hw0 + k) % RP, R - 1);
#pragma unroll
    for (int s = 0; s < KSN; ++s) {  // (steps past dk: zero here, the key fragment repeats the last step)
      qf[k][s] = ld128(qp + (size_t)(c * R + r) * p.dk + min(s, nst - 1) * 32);
      if (s >= nst) qf[k][s] = make_uint4(0, 0, 0, 0);
    }
  }
  uint4 tf[C::MT];                                                   // talk, A operand (both mixing steps use it)
#pragma unroll
  for (int mt = 0; mt < C::MT; ++mt) tf[mt] = reinterpret_cast<const uint4*>(pp.talk_frag)[mt * 64 + lane];
  __syncthreads();
#pragma unroll
  for (int k = 0; k < HW; ++k) ls[k] = lse[(hw0 + k) * 16 + rl];
  const unsigned klane = rl * p.dk + b * 8;                          // (scalar tile base + one lane offset)
  auto load_k = [&](uint4 (&kf)[C::NCW][2][KSN], int it) {
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int ts = __builtin_amdgcn_readfirstlane(btab[min(it * KT + tw0 + u, v.n - 1)]);
      const u16* kp = reinterpret_cast<const u16*>(p.k) + (int64_t)(ts >> lb) * p.k_sb + (ts & lm) * kTile * p.dk;
#pragma unroll
      for (int c = 0; c < C::NCW; ++c)
#pragma unroll
        for (int s = 0; s < KSN; ++s)
          kf[c][u][s] = ld128(kp + (int64_t)min(hw0 / RP + c, p.G - 1) * p.k_sh + min(s, nst - 1) * 32 + klane);
    }
  };
  // value tiles of a wave in chunks of NC; a step is one chunk of one 32-key group
  const int ndv = p.dv >> 4, nvt = p.G * ndv, nvw = (nvt + kPW - 1) / kPW, v0 = w * nvw;
  constexpr int NC = C::NC, CH = NV / NC, STEPS = KG * CH;
  static_assert(NV % NC == 0, "whole chunks");
  // (value tiles past the last compute something nobody stores)
  auto tile_at = [&](int u) { return min(v0 + min(u, nvw - 1), nvt - 1); };
  const u16* vbase = reinterpret_cast<const u16*>(p.v) + rl * p.block_size + (b & 1) * 8;
  auto load_v = [&](uint4 (&vf)[NC], int it, int step) {
    const int ts = btab[min(it * KT + 2 * (step / CH) + (b >> 1), v.n - 1)];
    const u16* vp = vbase + (int64_t)(ts >> lb) * p.v_sb + (ts & lm) * kTile;
#pragma unroll
    for (int n = 0; n < NC; ++n) {
      const int idx = tile_at((step % CH) * NC + n);
      vf[n] = ld128(vp + (int64_t)(idx / ndv) * p.v_sh + (int64_t)(idx % ndv) * 16 * p.block_size);
    }
  };

  f32x4 acc[NV][RP] = {};
  uint4 kf[C::NCW][2][KSN];
  load_k(kf, it0);
  // The values of a round's first step (two steps when there are several: va, vb) are requested at the end
  // of the round before it, its keys after the scores of the round before it
  static_assert(STEPS == 1 || STEPS % 2 == 0, "register sets by step parity");
  uint4 va[NC], vb[NC];
  load_v(va, it0, 0);
  if (STEPS > 1) load_v(vb, it0, 1);
  for (int it = it0; it < it1; ++it) {
    // ---- scores -> hi / lo weights
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int t = it * KT + tw0 + u;
      const int key0 = tile_of(v, min(t, v.n - 1)) * kTile;
      const bool ok = t < v.n, full = ok && all_visible(pos0, pos1, key0, p.window, p.keep);
      bool vis[4] = {true, true, true, true};
      if (!full) {
#pragma unroll
        for (int i = 0; i < 4; ++i) vis[i] = ok && sees(qpos, key0 + 4 * b + i, p.window, p.keep);
      }
      float x[HW][4];
#pragma unroll
      for (int k = 0; k < HW; ++k) {
        f32x4 a = {};
#pragma unroll
        for (int s = 0; s < KSN; ++s) a = mfma16(as_bf16x8(kf[k / RP][u][s]), as_bf16x8(qf[k][s]), a);
#pragma unroll
        for (int i = 0; i < 4; ++i) x[k][i] = vis[i] ? __builtin_amdgcn_exp2f(a[i] * sl2 - ls[k]) : 0.f;
      }
      // head h, part (hi 0, lo 1) at byte: HT 32 part * 1024 + h / 8 block; 16 block 2 part + h / 8; 8 block
      // part; 4 block 0, element 4 part + h
      char* xw = xm + ((tw0 + u) * kTile + 4 * b) * KB + rl * 16 + (HX == 4 ? hw0 * 2 : (hw0 >> 3) * 256 + (hw0 & 7) * 2);
      constexpr int LO = HX == 32 ? 1024 : HX == 16 ? 512 : HX == 8 ? 256 : 8;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if constexpr (HW == 1) {
          const u16 hi = f2bf(x[0][i]);
          *reinterpret_cast<u16*>(xw + i * KB) = hi;
          *reinterpret_cast<u16*>(xw + i * KB + LO) = f2bf(x[0][i] - bf2f(hi));
        } else {
          unsigned hi[HW / 2], lo[HW / 2];
#pragma unroll
          for (int k = 0; k < HW; k += 2) {
            hi[k / 2] = pack2(x[k][i], x[k + 1][i]);
            lo[k / 2] = pack2(x[k][i] - __uint_as_float(hi[k / 2] << 16), x[k + 1][i] - __uint_as_float(hi[k / 2] & 0xffff0000u));
          }
          if constexpr (HW == 2) {
            *reinterpret_cast<unsigned*>(xw + i * KB) = hi[0];
            *reinterpret_cast<unsigned*>(xw + i * KB + LO) = lo[0];
          } else {
            *reinterpret_cast<uint2*>(xw + i * KB) = make_uint2(hi[0], hi[1]);
            *reinterpret_cast<uint2*>(xw + i * KB + LO) = make_uint2(lo[0], lo[1]);
          }
        }
      }
    }
    lds_sync();
    if (!C::LATE_K) load_k(kf, it + 1);
    // ---- mixing: keys 4 kq .. 4 kq + 3
#pragma unroll
    for (int u = 0; u < KT / 2; ++u) {
      const int kq = w + 8 * u;
#pragma unroll
      for (int mt = 0; mt < C::MT; ++mt) {
        f32x4 y[4];
#pragma unroll
        for (int g = 0; g < 4; ++g) {
          y[g] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int ks = 0; ks < C::KM; ++ks)
            y[g] = mfma16(as_bf16x8(tf[mt]), *reinterpret_cast<const bf16x8*>(xm + (4 * kq + g) * KB + ks * 1024 + lane * 16), y[g]);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int h = 16 * mt + 4 * b + e;
          if (HX >= 16 || h < HX)
            *reinterpret_cast<uint2*>(pm + h * HS + (((kq >> 1) * 16) + rl) * 16 + (kq & 1) * 8) =
                make_uint2(pack2(y[0][e], y[1][e]), pack2(y[2][e], y[3][e]));
        }
      }
    }
    lds_sync();
    // ---- values
    auto load_p = [&](uint4 (&pf)[RP], int c, int kg) {
#pragma unroll
      for (int r = 0; r < RP; ++r)
        pf[r] = *reinterpret_cast<const uint4*>(pm + (c * RP + r) * HS + ((kg * 4 + b) * 16 + rl) * 16);
    };
    uint4 pf[RP];
#pragma unroll
    for (int st = 0; st < STEPS; ++st) {
      const int kg = st / CH;
      if (kg > 0 && it * KT + 2 * kg >= v.n) break;
      uint4(&vc)[NC] = st & 1 ? vb : va;
#pragma unroll
      for (int n = 0; n < NC; ++n) {
        const int u = (st % CH) * NC + n;
        // (a kv head's mixed weights serve all of this wave's value tiles of it)
        if (u == 0 || (!ONE && tile_at(u) / ndv != tile_at(u - 1) / ndv)) load_p(pf, tile_at(u) / ndv, kg);
#pragma unroll
        for (int r = 0; r < RP; ++r) acc[u][r] = mfma16(as_bf16x8(vc[n]), as_bf16x8(pf[r]), acc[u][r]);
      }
      // the step after next (or the next round's) into the registers just used
      if (STEPS == 1) load_v(vc, it + 1, 0);
      else load_v(vc, st + 2 < STEPS ? it : it + 1, st + 2 < STEPS ? st + 2 : st + 2 - STEPS);
    }
    if (C::LATE_K) load_k(kf, it + 1);
  }
  if (nact > 1) {
    // ---- every split's sums out (sc1), a ticket, and the last one adds them in order
    constexpr int kWave = NV * RP * 64 * 16, kPart = kPW * kWave;     // bytes per wave / workgroup
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
      const float g = gate[(c * RP + r) * 16 + rl];
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

template <int GP, int RP, int NV, int KSN>
int64_t prefill_cfg(const TalkPrefillParams& p, hipStream_t st, Want want) {
  using C = PrefillCfg<GP, RP, NV, KSN>;
  static_assert(C::LDS <= kMaxLds - 64, "LDS");
  if (want == WANT_FIT) return 0;
  if (want == WANT_PART) return (int64_t)kPW * NV * RP * 256;
  const int R = p.a.H / p.a.G;
  constexpr int RB = RP < 4 ? RP : 4;
  hipLaunchKernelGGL((talk_lse_kernel<RB, KSN>), dim3(p.n_tiles * p.a.G, (R + RB - 1) / RB), dim3(256), 0, st, p);
  const dim3 grid(p.n_tiles, p.splits), block(kPW * 64);
  if constexpr (KSN == 4 && NV == GP) {  // (the usual sizes)
    const int ndv = p.a.dv >> 4, nvw = (p.a.G * ndv + kPW - 1) / kPW;
    if (ndv % nvw == 0) {
      hipLaunchKernelGGL((talk_prefill_kernel<GP, RP, NV, KSN, true>), grid, block, C::LDS, st, p);
      return 0;
    }
  }
  hipLaunchKernelGGL((talk_prefill_kernel<GP, RP, NV, KSN, false>), grid, block, C::LDS, st, p);
  return 0;
}

template <int GP, int RP>
int64_t prefill_sizes(const TalkPrefillParams& p, hipStream_t st, Want want) {
  constexpr int N1 = GP, N2 = 2 * GP;   // value tiles per wave: dv <= 128 / <= 256
  const int need = (p.a.G * (p.a.dv >> 4) + kPW - 1) / kPW;
  if (need <= N1) {
    if (p.a.dk <= 64) return prefill_cfg<GP, RP, N1, 2>(p, st, want);
    if (p.a.dk <= 128) return prefill_cfg<GP, RP, N1, 4>(p, st, want);
    return prefill_cfg<GP, RP, N1, 8>(p, st, want);
  }
  if constexpr (GP * RP <= 16) {
    if (need <= N2) {
      if (p.a.dk <= 64) return prefill_cfg<GP, RP, N2, 2>(p, st, want);
      if (p.a.dk <= 128) return prefill_cfg<GP, RP, N2, 4>(p, st, want);
      return prefill_cfg<GP, RP, N2, 8>(p, st, want);
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
  if (p.rows < 1 || p.G < 1 || p.H < 1 || p.H % p.G || p.block_size < kTile || (p.block_size & (p.block_size - 1)) || p.dk % 32 || p.dv % 16) return -1;
  if (p.window < 0 || p.keep < 0) return -2;
  if ((p.k_sh | p.k_sb | p.v_sh | p.v_sb | p.ldq) % 8) return -3;
  return 0;
}

template <class T>
int launch_rows(const TalkAttnParams& p, hipStream_t st) {
  const size_t lds = mix_lds<T>(p.H);
  if (lds > kMaxLds - 64) return -5;
  const dim3 grid(p.rows * p.G, p.nch, (p.H / p.G + 15) / 16), block(256);
  hipLaunchKernelGGL((talk_scores_kernel<T>), grid, block, 0, st, p);
  hipLaunchKernelGGL((talk_mix_kernel<T>), grid, block, lds, st, p);
  return (int)hipGetLastError();
}

}  // namespace

extern "C" int vwa_talk_attention(const TalkAttnParams* p, hipStream_t st) {
  const int rc = check_attn(*p);
  if (rc) return rc;
  if (p->nch < 1 || !p->s || !p->stat || !p->part || !p->counters) return -4;
  if ((int64_t)p->nch * p->H * p->dv * 4 >= (1ll << 31)) return -5;
  return p->f32 ? launch_rows<float>(*p, st) : launch_rows<u16>(*p, st);
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
  if (p->max_tiles < 1 || p->max_tiles > kTab) return -8;  // (the kernel keeps the tiles' places in LDS)
  if (p->a.f32 || p->n_tiles < 1 || !p->tiles || !p->talk_frag || !p->lse || p->splits < 1 || p->a.ldo % 4) return -6;
  if (p->splits > 1) {
    const int64_t part = dispatch_prefill(*p, st, WANT_PART);
    if (!p->part || !p->tickets || part < 0 || part * p->splits * 4 >= (1ll << 31)) return -7;
  }
  const int64_t r = dispatch_prefill(*p, st, WANT_LAUNCH);
  if (r) return (int)r;
  return (int)hipGetLastError();
}
