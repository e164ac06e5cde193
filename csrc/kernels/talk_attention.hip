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
//  2) prefill form (bf16): a workgroup per 16 consecutive queries, its waves owning key tiles in the
//     score pass (all heads of a tile in one wave's registers: the mixing is lane-local, talk read
//     through scalar loads) and (kv head, 16 value columns) tiles in the value pass; the mixed weights
//     pass between them through LDS in B-operand order.
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
constexpr int kMaxKS = 8;                   // 32-wide steps over the q / k dimensions (dk <= 256)

// GP, RP: kv heads and query heads per kv head in the padded head order h = c * RP + r
// NV: (kv head, 16 value columns) tiles per wave; NW waves; QL: query fragments in LDS (else read
// from the q rows, L1 / L2)
template <int GP, int RP, int NV, int NW, bool QL>
struct PrefillCfg {
  static constexpr int HT = GP * RP, KEYS = NW * kTile, KG = KEYS / 32;
  static constexpr int P_BYTES = HT * KEYS * 16 * 2;                 // mixed weights
  static constexpr int RED_BYTES = NW * HT * 16 * 2 * 4;             // statistics of the waves (before P is used)
  static constexpr int PR = P_BYTES > RED_BYTES ? P_BYTES : RED_BYTES;
  static size_t lds(int dk) { return PR + HT * 16 * 4 + kTab * 4 + (QL ? (size_t)HT * dk * 16 * 2 : 0); }
};

template <int GP, int RP, int NV, int NW, bool QL>
__global__ __launch_bounds__(NW * 64) void talk_prefill_kernel(TalkPrefillParams pp) {
  using C = PrefillCfg<GP, RP, NV, NW, QL>;
  constexpr int HT = C::HT;
  const TalkAttnParams& p = pp.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  char* pm = smem;                                                   // [HT][KG][4][16 q][16 B]
  float* red = reinterpret_cast<float*>(smem);                       // [NW][HT][16][2]
  float* lse = reinterpret_cast<float*>(smem + C::PR);               // [HT][16]
  int* btab = reinterpret_cast<int*>(lse + HT * 16);
  uint4* qs = reinterpret_cast<uint4*>(btab + kTab);                 // [HT][dk / 32][64]
  const int lane = lane_id(), w = threadIdx.x >> 6, rl = lane & 15, b = lane >> 4;
  const int bt = xcd_remap((int)blockIdx.x, pp.n_tiles);
  const int row0 = pp.tiles[2 * bt], nq = pp.tiles[2 * bt + 1];
  const int R = p.H / p.G, nst = p.dk >> 5;
  const int pos0 = p.positions[row0], seq = p.seq_ids[row0];
  const int qrow = row0 + min(rl, nq - 1), qpos = pos0 + min(rl, nq - 1);
  const Vis v = vis_tiles(pos0, pos0 + nq - 1, p.window, p.keep);
  const float sl2 = p.scale * kLog2e;
  const int* gtab = p.block_table + (int64_t)seq * p.table_stride;
  const int nblk = (pos0 + nq - 1) / p.block_size + 1;
  const bool tab = nblk <= kTab;
  if (tab)
    for (int i = threadIdx.x; i < nblk; i += NW * 64) btab[i] = gtab[i];
  const u16* qp = reinterpret_cast<const u16*>(p.q) + (size_t)qrow * p.ldq + b * 8;
  if constexpr (QL) {
    for (int u = w; u < p.H * nst; u += NW) {
      const int h = u / nst, s = u % nst;
      qs[((size_t)((h / R) * RP + h % R) * nst + s) * 64 + lane] = ld128(qp + (size_t)h * p.dk + s * 32);
    }
  }
  __syncthreads();
  auto blk_of = [&](int key) -> int64_t {
    const int i = key / p.block_size;
    return tab ? btab[i] : gtab[i];
  };
  auto load_k = [&](uint4 (&kf)[kMaxKS], int c, int key0) {
    const u16* kp = reinterpret_cast<const u16*>(p.k) + blk_of(key0) * p.k_sb + (int64_t)c * p.k_sh +
                    (int64_t)(key0 % p.block_size + rl) * p.dk + b * 8;
#pragma unroll
    for (int s = 0; s < kMaxKS; ++s)
      if (s < nst) kf[s] = ld128(kp + s * 32);
  };
  // S^T tile of head (c, r): lane = query rl, keys 4b .. 4b+3
  auto score = [&](const uint4 (&kf)[kMaxKS], int c, int r) {
    f32x4 a = {};
#pragma unroll
    for (int s = 0; s < kMaxKS; ++s)
      if (s < nst) {
        uint4 qf;
        if constexpr (QL) qf = qs[((size_t)(c * RP + r) * nst + s) * 64 + lane];
        else qf = ld128(qp + (size_t)(c * R + r) * p.dk + s * 32);
        a = mfma16(as_bf16x8(kf[s]), as_bf16x8(qf), a);
      }
    return a;
  };

  // ---- pass 1: per-lane running (max, sum) of every head over this wave's tiles
  {
    float m[HT], l[HT];
#pragma unroll
    for (int h = 0; h < HT; ++h) {
      m[h] = -INFINITY;
      l[h] = 0.f;
    }
    for (int t = w; t < v.n; t += NW) {
      const int key0 = tile_of(v, t) * kTile;
      bool vis[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) vis[i] = sees(qpos, key0 + 4 * b + i, p.window, p.keep);
#pragma unroll
      for (int c = 0; c < GP; ++c) {
        if (c >= p.G) break;
        uint4 kf[kMaxKS];
        load_k(kf, c, key0);
#pragma unroll
        for (int r = 0; r < RP; ++r) {
          if (r >= R) break;
          const f32x4 a = score(kf, c, r);
          float s[4];
#pragma unroll
          for (int i = 0; i < 4; ++i) s[i] = vis[i] ? a[i] * sl2 : -INFINITY;
          float& mh = m[c * RP + r];
          const float mn = fmaxf(fmaxf(mh, fmaxf(s[0], s[1])), fmaxf(s[2], s[3]));
          const float ms = mn == -INFINITY ? 0.f : mn;
          float x = l[c * RP + r] * __builtin_amdgcn_exp2f(mh - ms);
#pragma unroll
          for (int i = 0; i < 4; ++i) x += __builtin_amdgcn_exp2f(s[i] - ms);
          l[c * RP + r] = x;
          mh = mn;
        }
      }
    }
#pragma unroll
    for (int h = 0; h < HT; ++h) {
#pragma unroll
      for (int o = 16; o < 64; o <<= 1) {
        const float mo = __shfl_xor(m[h], o, 64), lo = __shfl_xor(l[h], o, 64);
        const float mn = fmaxf(m[h], mo), ms = mn == -INFINITY ? 0.f : mn;
        l[h] = l[h] * __builtin_amdgcn_exp2f(m[h] - ms) + lo * __builtin_amdgcn_exp2f(mo - ms);
        m[h] = mn;
      }
      if (b == 0) {
        red[((w * HT + h) * 16 + rl) * 2] = m[h];
        red[((w * HT + h) * 16 + rl) * 2 + 1] = l[h];
      }
    }
  }
  __syncthreads();
  for (int u = threadIdx.x; u < HT * 16; u += NW * 64) {
    float m = -INFINITY, s = 0.f;
#pragma unroll
    for (int i = 0; i < NW; ++i) m = fmaxf(m, red[(i * HT * 16 + u) * 2]);
#pragma unroll
    for (int i = 0; i < NW; ++i) {
      const float li = red[(i * HT * 16 + u) * 2 + 1];
      s += li > 0.f ? li * __builtin_amdgcn_exp2f(red[(i * HT * 16 + u) * 2] - m) : 0.f;
    }
    lse[u] = s > 0.f ? m + __log2f(s) : 0.f;
  }
  __syncthreads();

  // ---- pass 2
  f32x4 acc[NV][RP] = {};
  const int ndv = p.dv >> 4, nvt = p.G * ndv;
  for (int it = 0; it * NW < v.n; ++it) {
    const int t = it * NW + w;
    char* pw = pm + ((((w >> 1) * 4 + 2 * (w & 1) + (b >> 1)) * 16 + rl) * 16) + (b & 1) * 8;
    constexpr int HS = C::KG * 4 * 16 * 16;  // bytes per head
    if (t < v.n) {
      const int key0 = tile_of(v, t) * kTile;
      bool vis[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) vis[i] = sees(qpos, key0 + 4 * b + i, p.window, p.keep);
      float x[HT][4];
#pragma unroll
      for (int c = 0; c < GP; ++c) {
        uint4 kf[kMaxKS];
        if (c < p.G) load_k(kf, c, key0);
#pragma unroll
        for (int r = 0; r < RP; ++r) {
          f32x4 a = {};
          const bool real = c < p.G && r < R;
          if (real) a = score(kf, c, r);
          const float ls = lse[(c * RP + r) * 16 + rl];
#pragma unroll
          for (int i = 0; i < 4; ++i)
            x[c * RP + r][i] = real && vis[i] ? __builtin_amdgcn_exp2f(a[i] * sl2 - ls) : 0.f;
        }
      }
#pragma unroll 1
      for (int h = 0; h < HT; ++h) {
        const float* tk = pp.talk_pad + h * HT;  // (uniform: scalar loads)
        float y[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int g = 0; g < HT; ++g) {
          const float tg = tk[g];
#pragma unroll
          for (int i = 0; i < 4; ++i) y[i] += tg * x[g][i];
        }
        *reinterpret_cast<uint2*>(pw + h * HS) = make_uint2(pack2(y[0], y[1]), pack2(y[2], y[3]));
      }
    } else {
#pragma unroll
      for (int h = 0; h < HT; ++h) *reinterpret_cast<uint2*>(pw + h * HS) = make_uint2(0u, 0u);
    }
    __syncthreads();
#pragma unroll
    for (int kg = 0; kg < C::KG; ++kg) {
      if (it * NW + 2 * kg >= v.n) break;
      const int tt = min(it * NW + 2 * kg + (b >> 1), v.n - 1);
      const int key = tile_of(v, tt) * kTile;
      const u16* vp = reinterpret_cast<const u16*>(p.v) + blk_of(key) * p.v_sb + (int64_t)rl * p.block_size +
                      key % p.block_size + (b & 1) * 8;
      uint4 vf[NV];
#pragma unroll
      for (int n = 0; n < NV; ++n) {
        const int idx = min(w + NW * n, nvt - 1);
        vf[n] = ld128(vp + (int64_t)(idx / ndv) * p.v_sh + (int64_t)(idx % ndv) * 16 * p.block_size);
      }
#pragma unroll
      for (int n = 0; n < NV; ++n) {
        const int idx = w + NW * n;
        if (idx >= nvt) break;
        const int c = idx / ndv;
#pragma unroll
        for (int r = 0; r < RP; ++r) {
          if (r >= R) break;
          const uint4 pf = *reinterpret_cast<const uint4*>(pm + (c * RP + r) * HS + ((kg * 4 + b) * 16 + rl) * 16);
          acc[n][r] = mfma16(as_bf16x8(vf[n]), as_bf16x8(pf), acc[n][r]);
        }
      }
    }
    __syncthreads();
  }
  // ---- gate, scale, store: lane (query rl, value columns 4b .. 4b+3 of the tile)
  if (rl >= nq) return;
#pragma unroll
  for (int n = 0; n < NV; ++n) {
    const int idx = w + NW * n;
    if (idx >= nvt) break;
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

template <int GP, int RP, int NV, int NW, bool QL>
int launch_prefill(const TalkPrefillParams& p, hipStream_t st) {
  hipLaunchKernelGGL((talk_prefill_kernel<GP, RP, NV, NW, QL>), dim3(p.n_tiles), dim3(NW * 64),
                     (PrefillCfg<GP, RP, NV, NW, QL>::lds(p.a.dk)), st, p);
  return 0;
}

// launch = null: only whether these sizes have an instantiation
template <int GP, int RP>
int prefill_sizes(const TalkPrefillParams& p, hipStream_t st, bool launch) {
  constexpr int HT = GP * RP;
  constexpr int NW = HT > 16 ? 4 : 8;       // 32 heads: 4 waves with twice the registers
  constexpr int N1 = (GP * 8 + NW - 1) / NW, N2 = (GP * 16 + NW - 1) / NW;   // dv <= 128 / <= 256
  const int need = (p.a.G * (p.a.dv >> 4) + NW - 1) / NW;
  const bool ql = PrefillCfg<GP, RP, N1, NW, true>::lds(p.a.dk) <= kMaxLds;
  if (need <= N1) {
    if (!launch) return 0;
    return ql ? launch_prefill<GP, RP, N1, NW, true>(p, st) : launch_prefill<GP, RP, N1, NW, false>(p, st);
  }
  if constexpr (HT <= 16) {
    if (need <= N2) {
      if (!launch) return 0;
      return ql ? launch_prefill<GP, RP, N2, NW, true>(p, st) : launch_prefill<GP, RP, N2, NW, false>(p, st);
    }
  }
  return -10;
}

int dispatch_prefill(const TalkPrefillParams& p, hipStream_t st, bool launch) {
  const TalkAttnParams& a = p.a;
  if (a.H < 1 || a.G < 1 || a.H % a.G || a.dk % 32 || a.dk > 32 * kMaxKS || a.dv % 16 || a.dv < 16) return -10;
  switch (pow2_up(a.G) * 100 + pow2_up(a.H / a.G)) {
    case 101: return prefill_sizes<1, 1>(p, st, launch);
    case 102: return prefill_sizes<1, 2>(p, st, launch);
    case 104: return prefill_sizes<1, 4>(p, st, launch);
    case 108: return prefill_sizes<1, 8>(p, st, launch);
    case 201: return prefill_sizes<2, 1>(p, st, launch);
    case 202: return prefill_sizes<2, 2>(p, st, launch);
    case 204: return prefill_sizes<2, 4>(p, st, launch);
    case 208: return prefill_sizes<2, 8>(p, st, launch);
    case 401: return prefill_sizes<4, 1>(p, st, launch);
    case 402: return prefill_sizes<4, 2>(p, st, launch);
    case 404: return prefill_sizes<4, 4>(p, st, launch);
    case 408: return prefill_sizes<4, 8>(p, st, launch);
    case 801: return prefill_sizes<8, 1>(p, st, launch);
    case 802: return prefill_sizes<8, 2>(p, st, launch);
    case 804: return prefill_sizes<8, 4>(p, st, launch);
    case 1601: return prefill_sizes<16, 1>(p, st, launch);
    case 1602: return prefill_sizes<16, 2>(p, st, launch);
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

extern "C" int vwa_talk_prefill_fits(int H, int G, int dk, int dv) {
  TalkPrefillParams p{};
  p.a.H = H;
  p.a.G = G;
  p.a.dk = dk;
  p.a.dv = dv;
  return dispatch_prefill(p, nullptr, false) == 0;
}

extern "C" int vwa_talk_prefill(const TalkPrefillParams* p, hipStream_t st) {
  const int rc = check_attn(p->a);
  if (rc) return rc;
  if (p->a.f32 || p->n_tiles < 1 || !p->tiles || !p->talk_pad || p->GP != pow2_up(p->a.G) ||
      p->RP != pow2_up(p->a.H / p->a.G) || p->a.ldo % 4)
    return -6;
  const int r = dispatch_prefill(*p, st, true);
  if (r) return r;
  return (int)hipGetLastError();
}
