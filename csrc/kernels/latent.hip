// Latent attention: keys and values of every head are projections of one cached latent c (plus one rotated
// key part shared by the heads), so decoding works in latent space:
//   score = (W_uk^T q) . c + q_rot . k_rot,   out_h = W_uv (sum_j p_j c_j)
// and reads one [latent | rotated part] row per token for all heads.
//
//  latent_rows      : rotation of the queries, norm of the latent, cache write
//  head_linear      : a product per head (W_uk^T q; also fused with latent_rows: latent_qkv)
//  latent_attention : (row, 16 heads, key chunk) -> unnormalised latent sums + softmax statistics
//  latent_out       : chunks merged with the heads' sinks, W_uv, output gate
#include "mixer_kernels.h"
#include "mq_attention.h"
#include "stack_types.h"

using namespace vwa;

namespace {

constexpr size_t kMaxLds = 160 * 1024 - 2048;
constexpr float kLog2e = 1.4426950408889634f;

// ------------------------------------------------------------------------------------------ per-head products
constexpr int kHlTiles = 2;                          // 16-column tiles per wave
constexpr int kHlCols = 4 * kHlTiles * 16;           // columns per workgroup

// block b, columns from cg * kHlCols, rows from r0 (16 NT of them)
template <class T, int NT>
VWA_DEVICE void head_linear_wg(const HeadLinearParams& p, int b, int cg, int r0) {
  using M = MM<T>;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rl = lane & 15, g = lane >> 4;
  const int nt = p.N >> 4, t0 = (cg * 4 + w) * kHlTiles, steps = p.K / M::KS;
  if (t0 >= nt) return;
  auto row_of = [&](int r) { return p.row_list ? p.row_list[r] : r; };
  const T* xp[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
    xp[t] = reinterpret_cast<const T*>(p.x) + (size_t)row_of(min(r0 + 16 * t + rl, p.rows - 1)) * p.ldx + (size_t)b * p.xs + g * M::EPL;
  const uint4* wp[kHlTiles];
#pragma unroll
  for (int j = 0; j < kHlTiles; ++j)
    wp[j] = reinterpret_cast<const uint4*>(p.w) + ((size_t)b * nt + min(t0 + j, nt - 1)) * steps * 64 + lane;
  f32x4 acc[NT][kHlTiles] = {};
  constexpr int U = NT == 1 ? 4 : 2;                 // steps whose loads are in flight together
  for (int s0 = 0; s0 < steps; s0 += U) {
    uint4 a[U][NT], f[U][kHlTiles];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int s = min(s0 + u, steps - 1);
#pragma unroll
      for (int j = 0; j < kHlTiles; ++j) f[u][j] = wp[j][s * 64];
#pragma unroll
      for (int t = 0; t < NT; ++t) a[u][t] = *reinterpret_cast<const uint4*>(xp[t] + s * M::KS);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (s0 + u >= steps) break;
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int j = 0; j < kHlTiles; ++j) acc[t][j] = M::mma(a[u][t], f[u][j], acc[t][j]);
    }
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = r0 + 16 * t + 4 * g + i;
      if (r >= p.rows) continue;
#pragma unroll
      for (int j = 0; j < kHlTiles; ++j) {
        if (t0 + j >= nt) continue;
        const int c = b * p.ys + (t0 + j) * 16 + rl;
        stv(reinterpret_cast<T*>(p.y) + (size_t)row_of(r) * p.ldy + c, acc[t][j][i]);
      }
    }
}

template <class T, int NT>
__global__ __launch_bounds__(256) void head_linear_kernel(HeadLinearParams p) {
  const int cgs = (p.N + kHlCols - 1) / kHlCols;
  head_linear_wg<T, NT>(p, blockIdx.x / cgs, blockIdx.x % cgs, blockIdx.y * 16 * NT);
}

// ------------------------------------------------------------------------------------------ row part
template <class T>
VWA_DEVICE void latent_row(const LatentRowsParams& p, int row) {
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const T* x = reinterpret_cast<const T*>(p.x) + (size_t)row * p.ldx;
  const int pos = min(max(p.positions[row], 0), p.max_pos - 1);
  const int64_t slot = p.slots[row];
  const int half = p.rot >> 1, hq = p.dim_p + p.rot_p;
  const float* cs = p.rope + (size_t)pos * p.rot;
  // rotated part of one head at src -> dst: pair (i, i + half) by thread i < half, the padding by the others
  auto rotate = [&](const T* src, T* dst, int i) {
    if (i < half) {
      const float u = ldv(src + i), v = ldv(src + i + half), c = cs[2 * i], s = cs[2 * i + 1];
      stv(dst + i, u * c - v * s);
      stv(dst + i + half, v * c + u * s);
    } else {
      const int e = p.rot + i - half;                // (padding columns)
      if (e < p.rot_p) dst[e] = src[e];
    }
  };
  const int units = half + p.rot_p - p.rot;
  T* q = reinterpret_cast<T*>(p.q_out) + (size_t)row * p.ldq + p.q_at;
  for (int u = tid; u < p.H * units; u += 256) {
    const int h = u / units, i = u % units;
    rotate(x + h * hq + p.dim_p, q + (size_t)h * p.q_head, i);
  }
  if (!p.has_kv || slot < 0) return;
  const T* c = x + p.H * hq;
  T* dst = reinterpret_cast<T*>(p.cache) + (slot / p.block_size) * p.c_sb + (slot % p.block_size) * (int64_t)(p.rank_p + p.rot_p);
  float ss = 0.f;
  for (int i = tid; i < p.rank; i += 256) {
    const float v = ldv(c + i);
    ss += v * v;
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float rs = 1.f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)p.rank + p.eps);
  for (int i = tid; i < p.rank_p; i += 256) stv(dst + i, i < p.rank ? ldv(c + i) * rs * p.norm[i] : 0.f);
  for (int i = tid; i < units; i += 256) rotate(c + p.rank_p, dst + p.rank_p, i);
}

template <class T>
__global__ __launch_bounds__(256) void latent_rows_kernel(LatentRowsParams p) {
  latent_row<T>(p, blockIdx.x);
}

// workgroups 0 .. n_lin - 1: products, the others: rows
template <class T, int NT>
__global__ __launch_bounds__(256) void latent_qkv_kernel(LatentRowsParams p, HeadLinearParams q, int n_lin) {
  if ((int)blockIdx.x < n_lin) {
    const int cgs = (q.N + kHlCols - 1) / kHlCols, per = q.nb * cgs;
    const int u = blockIdx.x % per;
    head_linear_wg<T, NT>(q, u / cgs, u % cgs, (blockIdx.x / per) * 16 * NT);
  } else {
    latent_row<T>(p, blockIdx.x - n_lin);
  }
}

// ------------------------------------------------------------------------------------------ attention, rows form
// 4 waves walk the chunk 64 keys at a time: scores by a wave per 16 keys x 16 heads, the weights pass between the
// waves in LDS in B-operand order, a wave owns NT 16-column value tiles.
constexpr int kKeys = 64;

struct Item {                                        // one workgroup's work
  int ri, row, h0, Hb, pos, t_beg, t_end;
  const int* table;
  float* stat;
};
// false: no key in the chunk (its statistics say so)
VWA_DEVICE bool attn_item(const LatentAttnParams& p, Item& x) {
  const int hgs = (p.H + 15) / 16, chunk = blockIdx.y;
  x.ri = blockIdx.x / hgs;
  x.h0 = (blockIdx.x % hgs) * 16;
  x.row = p.row_list ? p.row_list[x.ri] : x.ri;
  x.Hb = min(16, p.H - x.h0);
  x.pos = p.slots[x.row] >= 0 ? p.positions[x.row] : -1;
  x.table = p.block_table + (int64_t)p.seq_ids[x.row] * p.table_stride;
  const int nt = x.pos >= 0 ? x.pos / kKeys + 1 : 0, per = (nt + p.nch - 1) / p.nch;
  x.t_beg = chunk * per;
  x.t_end = min(nt, x.t_beg + per);
  x.stat = p.stat + (((size_t)x.ri * p.nch + chunk) * p.H + x.h0) * 2;
  if (x.t_beg < x.t_end) return true;
  if ((int)threadIdx.x < x.Hb) x.stat[2 * threadIdx.x] = x.stat[2 * threadIdx.x + 1] = 0.f;
  return false;
}

// online softmax of this round's scores (lane: keys key0 + 4 g + i, head rl): weights to pf, sums rescaled
template <class T, int NT>
VWA_DEVICE void attn_weights(const f32x4& sc_raw, float sl2, int key0, int pos, float (*s_max)[16], char* pf, float& m, float& l,
                             f32x4 (&acc)[NT]) {
  using M = MM<T>;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rl = lane & 15, g = lane >> 4;
  float sc[4], mx = -1e30f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    sc[i] = key0 + 16 * w + 4 * g + i <= pos ? sc_raw[i] * sl2 : -1e30f;
    mx = fmaxf(mx, sc[i]);
  }
  mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
  mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
  if (g == 0) s_max[w][rl] = mx;
  lds_sync();
  float mn = m;
#pragma unroll
  for (int i = 0; i < 4; ++i) mn = fmaxf(mn, s_max[i][rl]);
  const float alpha = __builtin_amdgcn_exp2f(m - mn);
  m = mn;
  l *= alpha;
  float pr[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    pr[i] = sc[i] > -1e30f ? __builtin_amdgcn_exp2f(sc[i] - mn) : 0.f;
    l += pr[i];
  }
  const int k = 16 * w + 4 * g, st = k / M::KS, kk = k % M::KS;
  st4(reinterpret_cast<T*>(pf + (st * 64 + 16 * (kk / M::EPL) + rl) * 16) + kk % M::EPL, pr);
#pragma unroll
  for (int n = 0; n < NT; ++n) acc[n] *= alpha;
  lds_sync();
}

template <int NT>
VWA_DEVICE void attn_finish(const LatentAttnParams& p, const Item& x, float m, float l, const f32x4 (&acc)[NT]) {
  __shared__ float s_sum[4][16];
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rl = lane & 15, g = lane >> 4, tid = threadIdx.x;
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (g == 0) s_sum[w][rl] = l;
  lds_sync();
  if (tid < x.Hb) {                                  // (every wave holds the same maximum; tid = head here)
    x.stat[2 * tid] = m;
    x.stat[2 * tid + 1] = (s_sum[0][tid] + s_sum[1][tid]) + (s_sum[2][tid] + s_sum[3][tid]);
  }
  if (rl >= x.Hb) return;
  float* part = p.part + (((size_t)x.ri * p.nch + blockIdx.y) * p.H + x.h0 + rl) * p.rank_p;
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int d = (w + 4 * n) * 16;
    if (d < p.rank_p) *reinterpret_cast<float4*>(part + d + 4 * g) = make_float4(acc[n][0], acc[n][1], acc[n][2], acc[n][3]);
  }
}

// bf16.  A wave's 16 keys lie in one cache block, one contiguous piece of dk / 32 KB-sized loads; the next round's
// are requested before this round's products.  The keys' rows go to LDS once and are read as the score product's
// A operand and, transposed (ds_read_tr), as the value product's.  SM: most 32-wide steps of dk; the queries'
// fragments stay in registers (QREG; else in LDS, and the keys are not requested ahead).
// (EXACT: dk is SM steps)
template <int NT, int SM, bool EXACT>
__global__ __launch_bounds__(256, 2) void latent_attn_kernel(LatentAttnParams p) {
  constexpr bool QREG = SM <= 20;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ float s_max[2][4][16];
  Item x;
  if (!attn_item(p, x)) return;
  const int dk = EXACT ? SM * 32 : p.rank_p + p.rot_p, steps = EXACT ? SM : dk >> 5, tid = threadIdx.x;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6), rl = lane & 15, g = lane >> 4;
  const int ks = dk * 2 + 16;
  char* pf = smem;                                   // [2][64][16 B]
  char* kt = smem + 2048;                            // [64 keys][ks]
  char* ql = kt + kKeys * ks;                        // (not QREG) [steps][64][16 B]
  const int lb = __builtin_ctz(p.block_size), cpr = dk >> 3;
  const u16* cache = reinterpret_cast<const u16*>(p.cache);
  const u16* qp = reinterpret_cast<const u16*>(p.q) + (size_t)x.row * p.ldq + (size_t)(x.h0 + min(rl, x.Hb - 1)) * dk + g * 8;
  uint4 qf[QREG ? SM : 1], nx[QREG ? SM : 1];
  const unsigned magic = ((1u << 20) + cpr - 1) / cpr;
  // this lane's i-th piece of the wave's 16 keys -> LDS (rows past pos, in the last tile, as zeros: whatever an
  // earlier owner of the block left there meets weights of zero)
  auto put = [&](int i, const uint4& v, int t) {
    const unsigned y = i * 64 + lane, r = (y * magic) >> 20;   // (y / cpr: y < 4096, cpr < 256)
    const bool live = t * kKeys + 16 * w + (int)r <= x.pos;
    *reinterpret_cast<uint4*>(kt + 16 * w * ks + (y + r) * 16) = live ? v : make_uint4(0, 0, 0, 0);  // (a row is cpr + 1 pieces apart)
  };
  auto tile_base = [&](int t) {                      // (a wave's keys past pos: the block of pos)
    const int key = min(t * kKeys + 16 * w, x.pos & ~15);
    return cache + (int64_t)x.table[key >> lb] * p.c_sb + (int64_t)(key & (p.block_size - 1)) * dk + lane * 8;
  };
  if constexpr (QREG) {
    const u16* kp = tile_base(x.t_beg);
#pragma unroll
    for (int i = 0; i < SM; ++i) nx[i] = ld128(kp + min(i, steps - 1) * 512);
#pragma unroll
    for (int i = 0; i < SM; ++i) qf[i] = ld128(qp + min(i, steps - 1) * 32);
  } else {
    for (int i = tid; i < steps * 64; i += 256)
      *reinterpret_cast<uint4*>(ql + i * 16) = ld128(reinterpret_cast<const u16*>(p.q) + (size_t)x.row * p.ldq +
                                                     (size_t)(x.h0 + min(i & 15, x.Hb - 1)) * dk + ((i >> 4) & 3) * 8 + (i >> 6) * 32);
  }
  const float sl2 = p.scale * kLog2e;
  float m = -1e30f, l = 0.f;
  f32x4 acc[NT] = {};
  for (int t = x.t_beg; t < x.t_end; ++t) {
    const int key0 = t * kKeys;
    if (t > x.t_beg) lds_sync();                     // (the previous keys and weights are read)
    if constexpr (QREG) {
#pragma unroll
      for (int i = 0; i < SM; ++i) put(min(i, steps - 1), nx[i], t);
      if (t + 1 < x.t_end) {
        const u16* kp = tile_base(t + 1);
#pragma unroll
        for (int i = 0; i < SM; ++i) nx[i] = ld128(kp + min(i, steps - 1) * 512);
      }
    } else {
      const u16* kp = tile_base(t);
      for (int i0 = 0; i0 < steps; i0 += 8) {
        uint4 v[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = ld128(kp + min(i0 + i, steps - 1) * 512);
#pragma unroll
        for (int i = 0; i < 8; ++i) put(min(i0 + i, steps - 1), v[i], t);
      }
    }
    lds_sync();
    // ---- scores of keys 16 w ..: D[key 4 g + i][head rl]
    f32x4 s[2] = {};
    const char* ka = kt + (16 * w + rl) * ks + g * 16;
    if constexpr (QREG) {
#pragma unroll
      for (int i = 0; i < SM; ++i)
        if (i < steps) s[i & 1] = mfma16(*reinterpret_cast<const bf16x8*>(ka + i * 64), as_bf16x8(qf[i]), s[i & 1]);
    } else {
      for (int i = 0; i < steps; ++i)
        s[0] = mfma16(*reinterpret_cast<const bf16x8*>(ka + i * 64), *reinterpret_cast<const bf16x8*>(ql + (i * 64 + lane) * 16), s[0]);
    }
    attn_weights<u16, NT>(s[0] + s[1], sl2, key0, x.pos, s_max[t & 1], pf, m, l, acc);
    // ---- latent sums: D[column 4 g + i][head rl]
#pragma unroll
    for (int st = 0; st < 2; ++st) {
      const bf16x8 pb = *reinterpret_cast<const bf16x8*>(pf + (st * 64 + lane) * 16);
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const int d = (w + 4 * n) * 16;
        if (d >= p.rank_p) continue;
        const unsigned char* a = reinterpret_cast<const unsigned char*>(kt) + (32 * st + 8 * g + (rl >> 2)) * ks + (d + 4 * (rl & 3)) * 2;
        const uint2 u = lds_tr16(a), v = lds_tr16(a + 4 * ks);
        acc[n] = mfma16(as_bf16x8(make_uint4(u.x, u.y, v.x, v.y)), pb, acc[n]);
      }
    }
  }
  attn_finish<NT>(p, x, m, l, acc);
}

// 32-bit: keys straight from the cache
template <int NT>
__global__ __launch_bounds__(256) void latent_attn_f32_kernel(LatentAttnParams p) {
  using M = MM<float>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ float s_max[2][4][16];
  Item x;
  if (!attn_item(p, x)) return;
  const int dk = p.rank_p + p.rot_p, steps = dk / M::KS, tid = threadIdx.x;
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6), rl = lane & 15, g = lane >> 4;
  char* pf = smem;                                   // [4][64][16 B]
  char* qf = smem + 4096;                            // [steps][64][16 B]
  for (int i = tid; i < steps * 64; i += 256) {
    const int s = i >> 6, ln = i & 63;
    const float* q = reinterpret_cast<const float*>(p.q) + (size_t)x.row * p.ldq + (size_t)(x.h0 + min(ln & 15, x.Hb - 1)) * dk;
    *reinterpret_cast<uint4*>(qf + i * 16) = *reinterpret_cast<const uint4*>(q + s * M::KS + (ln >> 4) * M::EPL);
  }
  const int lb = __builtin_ctz(p.block_size);
  const float* cache = reinterpret_cast<const float*>(p.cache);
  auto key_row = [&](int key) {                      // (keys past pos, in the last tile, repeat it)
    key = min(key, x.pos);
    return cache + (int64_t)x.table[key >> lb] * p.c_sb + (int64_t)(key & (p.block_size - 1)) * dk;
  };
  const float sl2 = p.scale * kLog2e;
  float m = -1e30f, l = 0.f;
  f32x4 acc[NT] = {};
  for (int t = x.t_beg; t < x.t_end; ++t) {
    const int key0 = t * kKeys;
    lds_sync();
    f32x4 s0 = {};
    const float* ka = key_row(key0 + 16 * w + rl) + g * M::EPL;
    for (int s = 0; s < steps; ++s)
      s0 = M::mma(*reinterpret_cast<const uint4*>(ka + s * M::KS), *reinterpret_cast<const uint4*>(qf + (s * 64 + lane) * 16), s0);
    attn_weights<float, NT>(s0, sl2, key0, x.pos, s_max[t & 1], pf, m, l, acc);
#pragma unroll
    for (int st = 0; st < kKeys / M::KS; ++st) {
      const uint4 pb = *reinterpret_cast<const uint4*>(pf + (st * 64 + lane) * 16);
      const int k = key0 + 16 * st + 4 * g;
      const float *k0 = key_row(k) + rl, *k1 = key_row(k + 1) + rl, *k2 = key_row(k + 2) + rl, *k3 = key_row(k + 3) + rl;
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const int d = (w + 4 * n) * 16;
        if (d >= p.rank_p) continue;
        acc[n] = M::mma(make_uint4(__float_as_uint(k0[d]), __float_as_uint(k1[d]), __float_as_uint(k2[d]), __float_as_uint(k3[d])), pb, acc[n]);
      }
    }
  }
  attn_finish<NT>(p, x, m, l, acc);
}

// ------------------------------------------------------------------------------------------ merge + value projection
// A workgroup per (head, rb <= 16 rows, 64 value columns): 4 column tiles x 2 halves of the latent.  The weights' first
// fragments are requested ahead of the merge; few rows spread a merge over the threads by chunks as well.
constexpr int kOutThreads = 512, kOutPre = 8;
template <class T>
size_t out_lds(int rank_p, int nch) { return 16 * ((size_t)rank_p * sizeof(T) + 16) + 16 * (size_t)nch * 4 + kOutThreads * 16; }

template <class T>
__global__ __launch_bounds__(kOutThreads) void latent_out_kernel(LatentOutParams p, int rb) {
  using M = MM<T>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int h = blockIdx.x, r0 = blockIdx.y * rb, tid = threadIdx.x, nr = min(rb, p.rows - r0);
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6), rl = lane & 15, g = lane >> 4;
  const int stride = p.rank_p * (int)sizeof(T) + 16;
  float4* red = reinterpret_cast<float4*>(smem + 16 * stride);               // [512]
  float* fac = reinterpret_cast<float*>(smem + 16 * stride + kOutThreads * 16);  // [16][nch]: weight of every chunk's sums
  const size_t cs = (size_t)p.H * p.rank_p;
  // ---- this wave's weights: column tile t, steps s0 .. s1
  const int steps = p.rank_p / M::KS, nt = p.vd >> 4, t = blockIdx.z * 4 + (w & 3), hs = (steps + 1) / 2;
  const int s0 = (w >> 2) * hs, s1 = min(steps, s0 + hs);
  const uint4* wp = reinterpret_cast<const uint4*>(p.w) + ((size_t)h * nt + min(t, nt - 1)) * steps * 64 + lane;
  uint4 wf[kOutPre];
#pragma unroll
  for (int i = 0; i < kOutPre; ++i) wf[i] = wp[min(s0 + i, steps - 1) * 64];
  // ---- chunk factors: 32 lanes per row
  {
    const int r = tid >> 5, k0 = tid & 31;
    if (r < nr) {
      const float2* st = reinterpret_cast<const float2*>(p.stat) + (size_t)(r0 + r) * p.nch * p.H + h;
      const float sink = p.sink[h] * kLog2e;
      float mx = sink;
      for (int k = k0; k < p.nch; k += 32) {
        const float2 v = st[(size_t)k * p.H];
        if (v.y > 0.f) mx = fmaxf(mx, v.x);
      }
#pragma unroll
      for (int o = 16; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 32));
      float sum = 0.f;
      for (int k = k0; k < p.nch; k += 32) {
        const float2 v = st[(size_t)k * p.H];
        const float e = v.y > 0.f ? __builtin_amdgcn_exp2f(v.x - mx) : 0.f;
        fac[r * p.nch + k] = e;
        sum += v.y * e;
      }
#pragma unroll
      for (int o = 16; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 32);
      const float inv = 1.f / (sum + __builtin_amdgcn_exp2f(sink - mx));
      for (int k = k0; k < p.nch; k += 32) fac[r * p.nch + k] *= inv;
    }
  }
  __syncthreads();
  // ---- merged sums -> LDS (T).  (An empty chunk's sums are not written: they count as zero.)
  const int quads = p.rank_p / 4, items = nr * quads, P = items < kOutThreads ? kOutThreads / items : 1;
  for (int i = tid; i < items * P; i += kOutThreads) {
    const int q = i % items, part = i / items, r = q / quads, d = (q % quads) * 4;
    const float* pt = p.part + ((size_t)(r0 + r) * p.nch * p.H + h) * p.rank_p + d;
    float v[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k = part; k < p.nch; k += 8 * P) {
      float u[8][4], f[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int kk = min(k + e * P, p.nch - 1);
        ld4(pt + (size_t)kk * cs, u[e]);
        f[e] = k + e * P < p.nch ? fac[r * p.nch + kk] : 0.f;
      }
#pragma unroll
      for (int e = 0; e < 8; ++e)
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] += f[e] > 0.f ? f[e] * u[e][j] : 0.f;
    }
    if (P == 1) st4(reinterpret_cast<T*>(smem + r * stride) + d, v);
    else red[i] = make_float4(v[0], v[1], v[2], v[3]);
  }
  if (P > 1) {
    __syncthreads();
    if (tid < items) {
      float v[4] = {0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k < P; ++k) {
        const float4 u = red[k * items + tid];
        v[0] += u.x;
        v[1] += u.y;
        v[2] += u.z;
        v[3] += u.w;
      }
      st4(reinterpret_cast<T*>(smem + (tid / quads) * stride) + (tid % quads) * 4, v);
    }
  }
  __syncthreads();
  const char* xa = smem + min(rl, nr - 1) * stride + g * 16;
  f32x4 a0 = {};
  for (int s = s0; s < s1; s += kOutPre) {
#pragma unroll
    for (int i = 0; i < kOutPre; ++i)
      if (s + i < s1) a0 = M::mma(*reinterpret_cast<const uint4*>(xa + (s + i) * 64), wf[i], a0);
    if (s + kOutPre < s1) {
#pragma unroll
      for (int i = 0; i < kOutPre; ++i) wf[i] = wp[min(s + kOutPre + i, steps - 1) * 64];
    }
  }
  f32x4* half = reinterpret_cast<f32x4*>(red);       // (the partial sums are read)
  if (w >= 4) half[(w & 3) * 64 + lane] = a0;
  __syncthreads();
  if (w >= 4 || t >= nt) return;
  a0 += half[w * 64 + lane];
  const int c = h * p.vd + t * 16 + rl;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 4 * g + i;
    if (r >= nr) continue;
    const int row = p.row_list ? p.row_list[r0 + r] : r0 + r;
    const float gt = sigm(ldv(reinterpret_cast<const T*>(p.gate) + (size_t)row * p.ldg + c));
    stv(reinterpret_cast<T*>(p.out) + (size_t)row * p.ldo + c, p.slots[row] < 0 ? 0.f : a0[i] * gt);
  }
}

int check_rows(const LatentRowsParams& p) {
  if (p.rows < 1 || p.H < 1 || p.rot < 2 || p.rot % 2 || p.rot_p < p.rot || p.rank < 1 || p.rank_p < p.rank || p.max_pos < 1 ||
      p.block_size < 1)
    return -1;
  return 0;
}
int check_lin(const HeadLinearParams& p) {
  if (p.rows < 1 || p.nb < 1 || p.N < 16 || p.N % 16 || p.K < 32 || p.K % 32 || p.ldx % 8 || p.xs % 8) return -2;
  if ((reinterpret_cast<uintptr_t>(p.x) | reinterpret_cast<uintptr_t>(p.w)) & 15) return -3;
  return 0;
}

template <class T>
void launch_head_linear(const HeadLinearParams& p, hipStream_t st) {
  const int cgs = (p.N + kHlCols - 1) / kHlCols;
  if (p.rows <= 16)
    hipLaunchKernelGGL((head_linear_kernel<T, 1>), dim3(p.nb * cgs, 1), dim3(256), 0, st, p);
  else
    hipLaunchKernelGGL((head_linear_kernel<T, 4>), dim3(p.nb * cgs, (p.rows + 63) / 64), dim3(256), 0, st, p);
}

template <class T>
void launch_qkv(const LatentRowsParams& p, const HeadLinearParams& q, hipStream_t st) {
  const int cgs = (q.N + kHlCols - 1) / kHlCols, per = q.nb * cgs;
  if (q.rows <= 16) {
    hipLaunchKernelGGL((latent_qkv_kernel<T, 1>), dim3(per + p.rows), dim3(256), 0, st, p, q, per);
  } else {
    const int n = per * ((q.rows + 63) / 64);
    hipLaunchKernelGGL((latent_qkv_kernel<T, 4>), dim3(n + p.rows), dim3(256), 0, st, p, q, n);
  }
}

template <int NT, int SM, bool EXACT>
int launch_attn_bf16(const LatentAttnParams& p, hipStream_t st) {
  const int dk = p.rank_p + p.rot_p;
  const size_t lds = 2048 + (size_t)kKeys * (dk * 2 + 16) + (SM <= 20 ? 0 : (size_t)dk * 32);
  if (lds > kMaxLds) return -10;
  hipLaunchKernelGGL((latent_attn_kernel<NT, SM, EXACT>), dim3(p.rows * ((p.H + 15) / 16), p.nch), dim3(256), lds, st, p);
  return (int)hipGetLastError();
}
int launch_attn(const LatentAttnParams& p, hipStream_t st) {
  const int per = (p.rank_p / 16 + 3) / 4, steps = (p.rank_p + p.rot_p) / 32;  // value tiles per wave
  if (per <= 2 && steps <= 8) return launch_attn_bf16<2, 8, false>(p, st);
  if (per <= 4 && steps <= 12) return launch_attn_bf16<4, 12, false>(p, st);
  if (per <= 8 && steps == 18) return launch_attn_bf16<8, 18, true>(p, st);
  if (per <= 8 && steps <= 20) return launch_attn_bf16<8, 20, false>(p, st);
  if (per <= 16 && steps <= 60) return launch_attn_bf16<16, 60, false>(p, st);
  return -10;
}
template <int NT>
int launch_attn_f32(const LatentAttnParams& p, hipStream_t st) {
  const size_t lds = 4096 + (size_t)(p.rank_p + p.rot_p) * 64;
  if (lds > kMaxLds) return -10;
  hipLaunchKernelGGL((latent_attn_f32_kernel<NT>), dim3(p.rows * ((p.H + 15) / 16), p.nch), dim3(256), lds, st, p);
  return (int)hipGetLastError();
}

}  // namespace

extern "C" int vwa_head_linear(const HeadLinearParams* p, hipStream_t st) {
  const int rc = check_lin(*p);
  if (rc) return rc;
  p->f32 ? launch_head_linear<float>(*p, st) : launch_head_linear<u16>(*p, st);
  return (int)hipGetLastError();
}

extern "C" int vwa_latent_rows(const LatentRowsParams* p, hipStream_t st) {
  const int rc = check_rows(*p);
  if (rc) return rc;
  if (p->f32) hipLaunchKernelGGL((latent_rows_kernel<float>), dim3(p->rows), dim3(256), 0, st, *p);
  else hipLaunchKernelGGL((latent_rows_kernel<u16>), dim3(p->rows), dim3(256), 0, st, *p);
  return (int)hipGetLastError();
}

extern "C" int vwa_latent_qkv(const LatentRowsParams* p, const HeadLinearParams* q, hipStream_t st) {
  const int rc = check_rows(*p) ? check_rows(*p) : check_lin(*q);
  if (rc) return rc;
  p->f32 ? launch_qkv<float>(*p, *q, st) : launch_qkv<u16>(*p, *q, st);
  return (int)hipGetLastError();
}

extern "C" int vwa_latent_attention(const LatentAttnParams* p, hipStream_t st) {
  if (p->rows < 1 || p->H < 1 || p->rank_p % 32 || p->rot_p % 32 || p->rank_p < 32 || p->nch < 1 || p->block_size < 16 ||
      (p->block_size & (p->block_size - 1)) || p->ldq % 8 || !p->part || !p->stat)
    return -1;
  if (!p->f32) return launch_attn(*p, st);
  return p->rank_p <= 128 ? launch_attn_f32<2>(*p, st) : p->rank_p <= 512 ? launch_attn_f32<8>(*p, st)
         : p->rank_p <= 1024 ? launch_attn_f32<16>(*p, st) : -10;
}

extern "C" int vwa_latent_out(const LatentOutParams* p, hipStream_t st) {
  if (p->rows < 1 || p->H < 1 || p->vd % 16 || p->rank_p % 32 || p->nch < 1 || !p->part || !p->stat || !p->sink) return -1;
  const size_t lds = p->f32 ? out_lds<float>(p->rank_p, p->nch) : out_lds<u16>(p->rank_p, p->nch);
  if (lds > kMaxLds) return -10;
  // (the merges are the work: fewer rows each while the launch is short of workgroups)
  int rb = 16;
  while (rb > 2 && p->H * ((p->vd + 63) / 64) * ((p->rows + rb - 1) / rb) < 256) rb /= 2;
  const dim3 grid(p->H, (p->rows + rb - 1) / rb, (p->vd + 63) / 64), block(kOutThreads);
  if (p->f32) hipLaunchKernelGGL((latent_out_kernel<float>), grid, block, lds, st, *p, rb);
  else hipLaunchKernelGGL((latent_out_kernel<u16>), grid, block, lds, st, *p, rb);
  return (int)hipGetLastError();
}
