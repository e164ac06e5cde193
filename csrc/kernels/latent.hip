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
#pragma unroll 4
  for (int s = 0; s < steps; ++s) {
    uint4 a[NT], f[kHlTiles];
#pragma unroll
    for (int j = 0; j < kHlTiles; ++j) f[j] = wp[j][s * 64];
#pragma unroll
    for (int t = 0; t < NT; ++t) a[t] = *reinterpret_cast<const uint4*>(xp[t] + s * M::KS);
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int j = 0; j < kHlTiles; ++j) acc[t][j] = M::mma(a[t], f[j], acc[t][j]);
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
// 4 waves walk the chunk 64 keys at a time.  bf16: the keys' rows are staged in LDS once, read as the score
// product's A operand and, transposed (ds_read_tr), as the value product's.  Scores: a wave per 16 keys x 16
// heads.  The weights pass between the waves in LDS in B-operand order; a wave owns NT 16-column value tiles.
constexpr int kKeys = 64;

template <class T> VWA_DEVICE int key_stride(int dk) { return dk * (int)sizeof(T) + 16; }
template <class T>
size_t attn_lds(int dk) {
  return (size_t)dk / MM<T>::KS * 1024 + kKeys * 16 * sizeof(T) + (sizeof(T) == 2 ? (size_t)kKeys * (dk * 2 + 16) : 0);
}

template <class T, int NT>
__global__ __launch_bounds__(256) void latent_attn_kernel(LatentAttnParams p) {
  using M = MM<T>;
  constexpr bool BF = sizeof(T) == 2;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ float s_max[2][4][16], s_sum[4][16];
  const int hgs = (p.H + 15) / 16, ri = blockIdx.x / hgs, h0 = (blockIdx.x % hgs) * 16, chunk = blockIdx.y;
  const int row = p.row_list ? p.row_list[ri] : ri;
  const int Hb = min(16, p.H - h0), dk = p.rank_p + p.rot_p, steps = dk / M::KS, tid = threadIdx.x;
  const bool live = p.slots[row] >= 0;
  const int pos = live ? p.positions[row] : -1, seq = p.seq_ids[row];
  const int nt = pos >= 0 ? pos / kKeys + 1 : 0, per = (nt + p.nch - 1) / p.nch;
  const int t_beg = chunk * per, t_end = min(nt, t_beg + per);
  float* stat = p.stat + (((size_t)ri * p.nch + chunk) * p.H + h0) * 2;
  if (t_beg >= t_end) {
    if (tid < Hb) stat[2 * tid] = stat[2 * tid + 1] = 0.f;
    return;
  }
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6), rl = lane & 15, g = lane >> 4;
  char* qf = smem;                                   // [steps][64][16 B]
  char* pf = smem + steps * 1024;                    // [64 / KS][64][16 B]
  char* kt = pf + kKeys * 16 * sizeof(T);            // (bf16) [64][key_stride]
  const int ks = key_stride<T>(dk);
  for (int i = tid; i < steps * 64; i += 256) {
    const int s = i >> 6, l = i & 63;
    const T* q = reinterpret_cast<const T*>(p.q) + (size_t)row * p.ldq + (size_t)(h0 + min(l & 15, Hb - 1)) * dk;
    *reinterpret_cast<uint4*>(qf + i * 16) = *reinterpret_cast<const uint4*>(q + s * M::KS + (l >> 4) * M::EPL);
  }
  const int lb = __builtin_ctz(p.block_size);
  const int* table = p.block_table + (int64_t)seq * p.table_stride;
  const T* cache = reinterpret_cast<const T*>(p.cache);
  auto key_row = [&](int key) {                      // (keys past pos, in the last tile, repeat it)
    key = min(key, pos);
    return cache + (int64_t)table[key >> lb] * p.c_sb + (int64_t)(key & (p.block_size - 1)) * dk;
  };
  const float sl2 = p.scale * kLog2e;
  float m = -1e30f, l = 0.f;
  f32x4 acc[NT] = {};
  const int ndv = p.rank_p >> 4;
  for (int t = t_beg; t < t_end; ++t) {
    const int key0 = t * kKeys;
    __syncthreads();                                 // (the previous keys and weights are read)
    if constexpr (BF) {
      const int cpr = dk / 8;                        // 16-byte pieces per key
#pragma unroll 6
      for (int i = tid; i < kKeys * cpr; i += 256) {
        const int r = i / cpr, c = i % cpr;
        *reinterpret_cast<uint4*>(kt + r * ks + c * 16) = ld128(reinterpret_cast<const u16*>(key_row(key0 + r)) + c * 8);
      }
      __syncthreads();
    }
    // ---- scores of keys 16 w ..: D[key 4 g + i][head rl]
    f32x4 s0 = {}, s1 = {};
    if constexpr (BF) {
      const char* ka = kt + (16 * w + rl) * ks + g * 16;
      int s = 0;
      for (; s + 1 < steps; s += 2) {
        s0 = M::mma(*reinterpret_cast<const uint4*>(ka + s * 64), *reinterpret_cast<const uint4*>(qf + (s * 64 + lane) * 16), s0);
        s1 = M::mma(*reinterpret_cast<const uint4*>(ka + s * 64 + 64), *reinterpret_cast<const uint4*>(qf + (s * 64 + 64 + lane) * 16), s1);
      }
      if (s < steps) s0 = M::mma(*reinterpret_cast<const uint4*>(ka + s * 64), *reinterpret_cast<const uint4*>(qf + (s * 64 + lane) * 16), s0);
    } else {
      const T* ka = key_row(key0 + 16 * w + rl) + g * M::EPL;
      for (int s = 0; s < steps; ++s)
        s0 = M::mma(*reinterpret_cast<const uint4*>(ka + s * M::KS), *reinterpret_cast<const uint4*>(qf + (s * 64 + lane) * 16), s0);
    }
    float sc[4], mx = -1e30f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      sc[i] = key0 + 16 * w + 4 * g + i <= pos ? (s0[i] + s1[i]) * sl2 : -1e30f;
      mx = fmaxf(mx, sc[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (g == 0) s_max[t & 1][w][rl] = mx;
    __syncthreads();
    float mn = m;
#pragma unroll
    for (int i = 0; i < 4; ++i) mn = fmaxf(mn, s_max[t & 1][i][rl]);
    const float alpha = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    l *= alpha;
    float pr[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      pr[i] = sc[i] > -1e30f ? __builtin_amdgcn_exp2f(sc[i] - mn) : 0.f;
      l += pr[i];
    }
    // weights of 4 consecutive keys in B-operand order
    {
      const int k = 16 * w + 4 * g, st = k / M::KS, kk = k % M::KS;
      st4(reinterpret_cast<T*>(pf + (st * 64 + 16 * (kk / M::EPL) + rl) * 16) + kk % M::EPL, pr);
    }
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[n] *= alpha;
    __syncthreads();
    // ---- latent sums: D[column 4 g + i][head rl]
#pragma unroll
    for (int st = 0; st < kKeys / M::KS; ++st) {
      const uint4 pb = *reinterpret_cast<const uint4*>(pf + (st * 64 + lane) * 16);
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const int d = (w + 4 * n) * 16;
        if (d >= p.rank_p) continue;
        uint4 v;
        if constexpr (BF) {
          const unsigned char* a = reinterpret_cast<const unsigned char*>(kt) + (32 * st + 8 * g + (rl >> 2)) * ks + (d + 4 * (rl & 3)) * 2;
          const uint2 lo = lds_tr16(a), hi = lds_tr16(a + 4 * ks);
          v = make_uint4(lo.x, lo.y, hi.x, hi.y);
        } else {
          const int k = key0 + 16 * st + 4 * g;
          v = make_uint4(__float_as_uint(key_row(k)[d + rl]), __float_as_uint(key_row(k + 1)[d + rl]),
                         __float_as_uint(key_row(k + 2)[d + rl]), __float_as_uint(key_row(k + 3)[d + rl]));
        }
        acc[n] = M::mma(v, pb, acc[n]);
      }
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (g == 0) s_sum[w][rl] = l;
  __syncthreads();
  if (tid < Hb) {
    stat[2 * tid] = m;                               // (every wave holds the same maximum; tid = head here)
    stat[2 * tid + 1] = (s_sum[0][tid] + s_sum[1][tid]) + (s_sum[2][tid] + s_sum[3][tid]);
  }
  if (rl >= Hb) return;
  float* part = p.part + (((size_t)ri * p.nch + chunk) * p.H + h0 + rl) * p.rank_p;
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int d = (w + 4 * n) * 16;
    if (d < ndv * 16) *reinterpret_cast<float4*>(part + d + 4 * g) = make_float4(acc[n][0], acc[n][1], acc[n][2], acc[n][3]);
  }
}

// ------------------------------------------------------------------------------------------ merge + value projection
constexpr int kOutWaves = 8;
template <class T>
size_t out_lds(int rank_p, int nch) { return 16 * ((size_t)rank_p * sizeof(T) + 16) + 16 * (size_t)nch * 4; }

template <class T>
__global__ __launch_bounds__(kOutWaves * 64) void latent_out_kernel(LatentOutParams p) {
  using M = MM<T>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int h = blockIdx.x, r0 = blockIdx.y * 16, tid = threadIdx.x, nr = min(16, p.rows - r0);
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6), rl = lane & 15, g = lane >> 4;
  const int stride = p.rank_p * (int)sizeof(T) + 16;
  float* fac = reinterpret_cast<float*>(smem + 16 * stride);   // [16][nch]: weight of every chunk's sums
  const size_t cs = (size_t)p.H * p.rank_p;
  // ---- chunk factors: 32 lanes per row
  {
    const int r = tid >> 5, k0 = tid & 31;
    if (r < nr) {
      const float* st = p.stat + ((size_t)(r0 + r) * p.nch * p.H + h) * 2;
      const float sink = p.sink[h] * kLog2e;
      float mx = sink;
      for (int k = k0; k < p.nch; k += 32)
        if (st[(size_t)k * p.H * 2 + 1] > 0.f) mx = fmaxf(mx, st[(size_t)k * p.H * 2]);
#pragma unroll
      for (int o = 16; o > 0; o >>= 1) mx = fmaxf(mx, __shfl_xor(mx, o, 32));
      float sum = 0.f;
      for (int k = k0; k < p.nch; k += 32) {
        const float l = st[(size_t)k * p.H * 2 + 1], e = l > 0.f ? __builtin_amdgcn_exp2f(st[(size_t)k * p.H * 2] - mx) : 0.f;
        fac[r * p.nch + k] = e;
        sum += l * e;
      }
#pragma unroll
      for (int o = 16; o > 0; o >>= 1) sum += __shfl_xor(sum, o, 32);
      const float inv = 1.f / (sum + __builtin_amdgcn_exp2f(sink - mx));
      for (int k = k0; k < p.nch; k += 32) fac[r * p.nch + k] *= inv;
    }
  }
  __syncthreads();
  const int quads = p.rank_p / 4;
  for (int i = tid; i < nr * quads; i += kOutWaves * 64) {
    const int r = i / quads, d = (i % quads) * 4;
    const float* pt = p.part + ((size_t)(r0 + r) * p.nch * p.H + h) * p.rank_p + d;
    float v[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k = 0; k < p.nch; ++k) {
      const float f = fac[r * p.nch + k];
      if (f == 0.f) continue;                        // (an empty chunk's sums are not written)
      float u[4];
      ld4(pt + (size_t)k * cs, u);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] += f * u[j];
    }
    st4(reinterpret_cast<T*>(smem + r * stride) + d, v);
  }
  __syncthreads();
  const int steps = p.rank_p / M::KS, nt = p.vd >> 4;
  for (int t = w; t < nt; t += kOutWaves) {
    const uint4* wp = reinterpret_cast<const uint4*>(p.w) + ((size_t)h * nt + t) * steps * 64 + lane;
    const char* xa = smem + min(rl, nr - 1) * stride + g * 16;
    f32x4 a0 = {}, a1 = {};
    int s = 0;
#pragma unroll 4
    for (; s + 1 < steps; s += 2) {
      a0 = M::mma(*reinterpret_cast<const uint4*>(xa + s * 64), wp[s * 64], a0);
      a1 = M::mma(*reinterpret_cast<const uint4*>(xa + s * 64 + 64), wp[s * 64 + 64], a1);
    }
    if (s < steps) a0 = M::mma(*reinterpret_cast<const uint4*>(xa + s * 64), wp[s * 64], a0);
    const int c = h * p.vd + t * 16 + rl;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 4 * g + i;
      if (r >= nr) continue;
      const int row = p.row_list ? p.row_list[r0 + r] : r0 + r;
      const float gt = sigm(ldv(reinterpret_cast<const T*>(p.gate) + (size_t)row * p.ldg + c));
      stv(reinterpret_cast<T*>(p.out) + (size_t)row * p.ldo + c, p.slots[row] < 0 ? 0.f : (a0[i] + a1[i]) * gt);
    }
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

template <class T, int NT>
int launch_attn_nt(const LatentAttnParams& p, hipStream_t st) {
  const size_t lds = attn_lds<T>(p.rank_p + p.rot_p);
  if (lds > kMaxLds) return -10;
  hipLaunchKernelGGL((latent_attn_kernel<T, NT>), dim3(p.rows * ((p.H + 15) / 16), p.nch), dim3(256), lds, st, p);
  return (int)hipGetLastError();
}
template <class T>
int launch_attn(const LatentAttnParams& p, hipStream_t st) {
  const int per = (p.rank_p / 16 + 3) / 4;           // value tiles per wave
  if (per <= 2) return launch_attn_nt<T, 2>(p, st);
  if (per <= 4) return launch_attn_nt<T, 4>(p, st);
  if (per <= 8) return launch_attn_nt<T, 8>(p, st);
  if (per <= 16) return launch_attn_nt<T, 16>(p, st);
  return -10;
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
  return p->f32 ? launch_attn<float>(*p, st) : launch_attn<u16>(*p, st);
}

extern "C" int vwa_latent_out(const LatentOutParams* p, hipStream_t st) {
  if (p->rows < 1 || p->H < 1 || p->vd % 16 || p->rank_p % 32 || p->nch < 1 || !p->part || !p->stat || !p->sink) return -1;
  const size_t lds = p->f32 ? out_lds<float>(p->rank_p, p->nch) : out_lds<u16>(p->rank_p, p->nch);
  if (lds > kMaxLds) return -10;
  const dim3 grid(p->H, (p->rows + 15) / 16), block(kOutWaves * 64);
  if (p->f32) hipLaunchKernelGGL((latent_out_kernel<float>), grid, block, lds, st, *p);
  else hipLaunchKernelGGL((latent_out_kernel<u16>), grid, block, lds, st, *p);
  return (int)hipGetLastError();
}
