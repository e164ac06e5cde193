// Routed experts.
//
//  moe_route : sigmoid router scores (MFMA, f32 sums), the best ``top`` experts of every row, and the pairs
//              (row, choice) grouped by expert into tiles of at most ``tile`` pairs -- by the last workgroup
//  moe_gemm  : the experts' matrices over such a tile (here tiles of 16 or 32 pairs, streaming; of 128 or 256
//              go to gemm.hip's grouped launch).  First launch: the tile's rows times gate and up, scaled
//              by the pair's score ahead of the activation (w (W h) = W (w h)); second: down, one row per pair.
//              (The pairs of a row are added, in the order of its choices, by add_norm.)
// A row's results do not depend on the tile it lands in, so the order inside an expert is free.
#include "mixer_kernels.h"
#include "stack_types.h"
#include "vwa_kernels.h"

using namespace vwa;

namespace {

constexpr size_t kMaxLds = 160 * 1024 - 8192;
constexpr int kRouteWaves = 8, kRouteThreads = kRouteWaves * 64, kMaxExperts = 256;

// pairs -> tiles of one expert each (the whole workgroup); id_of(pair): its expert
template <class F>
VWA_DEVICE void group_pairs(const MoeRouteParams& p, F&& id_of) {
  __shared__ int cnt[kMaxExperts], first[kMaxExperts], s_total;
  const int tid = threadIdx.x, P = p.rows * p.top;
  for (int e = tid; e < p.E; e += kRouteThreads) cnt[e] = 0;
  __syncthreads();
  constexpr int B = 8;                               // ids whose loads are in flight together
  auto for_pairs = [&](auto&& fn) {
    for (int i0 = tid; i0 < P; i0 += B * kRouteThreads) {
      int e[B];
#pragma unroll
      for (int k = 0; k < B; ++k) e[k] = id_of(min(i0 + k * kRouteThreads, P - 1));
#pragma unroll
      for (int k = 0; k < B; ++k)
        if (i0 + k * kRouteThreads < P && e[k] >= 0) fn(i0 + k * kRouteThreads, e[k]);
    }
  };
  for_pairs([&](int, int e) { atomicAdd(&cnt[e], 1); });
  __syncthreads();
  if (tid < 64) {                                    // exclusive prefix of the experts' tile counts
    int base = 0;
    for (int e0 = 0; e0 < p.E; e0 += 64) {
      const int e = e0 + tid, n = e < p.E ? (cnt[e] + p.tile - 1) / p.tile : 0;
      int x = n;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int y = __shfl_up(x, o, 64);
        if (tid >= o) x += y;
      }
      if (e < p.E) first[e] = base + x - n;
      base += __shfl(x, 63, 64);
    }
    if (tid == 0) s_total = base;
  }
  __syncthreads();
  for (int e = tid; e < p.E; e += kRouteThreads) {
    const int n = cnt[e];
    for (int k = 0; k * p.tile < n; ++k) {
      int* t = p.tiles + 1 + 3 * (first[e] + k);
      t[0] = e;
      t[1] = (first[e] + k) * p.tile;
      t[2] = min(p.tile, n - k * p.tile);
    }
  }
  if (tid == 0) p.tiles[0] = s_total;
  __syncthreads();
  for (int e = tid; e < p.E; e += kRouteThreads) cnt[e] = first[e] * p.tile;
  __syncthreads();
  for_pairs([&](int i, int e) { p.order[atomicAdd(&cnt[e], 1)] = i; });
}

template <class T>
__global__ __launch_bounds__(kRouteThreads) void moe_route_kernel(MoeRouteParams p) {
  using M = MM<T>;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ int s_last;
  const int tid = threadIdx.x, lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6), rl = lane & 15, g = lane >> 4;
  const int r0 = blockIdx.x * 16, nr = min(16, p.rows - r0), et = (p.E + 15) / 16, Ep = et * 16, steps = p.K / M::KS;
  float* red = reinterpret_cast<float*>(smem);       // [waves][Ep][16 rows]
  float* sc = red + kRouteWaves * Ep * 16;           // [16 rows][Ep + 1]
  const T* h = reinterpret_cast<const T*>(p.h) + (size_t)(r0 + min(rl, nr - 1)) * p.ldh + g * M::EPL;
  const uint4* wf = reinterpret_cast<const uint4*>(p.w) + lane;
  const bool live = p.slots[r0 + min(tid >> 5, nr - 1)] >= 0;  // (of the row whose experts this thread chooses)
  for (int e = 0; e < et; ++e) {                     // D[expert 4 g + i][row rl], every wave a part of K
    f32x4 acc = {};
    for (int s0 = w; s0 < steps; s0 += 8 * kRouteWaves) {
      uint4 a[8], b[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int s = min(s0 + u * kRouteWaves, steps - 1);
        a[u] = wf[((size_t)e * steps + s) * 64];
        b[u] = *reinterpret_cast<const uint4*>(h + s * M::KS);
      }
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (s0 + u * kRouteWaves < steps) acc = M::mma(a[u], b[u], acc);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) red[(w * Ep + e * 16 + 4 * g + i) * 16 + rl] = acc[i];
  }
  __syncthreads();
  for (int i = tid; i < Ep * 16; i += kRouteThreads) {
    float z = 0.f;
#pragma unroll
    for (int k = 0; k < kRouteWaves; ++k) z += red[k * Ep * 16 + i];
    sc[(i & 15) * (Ep + 1) + (i >> 4)] = (i >> 4) < p.E ? 1.f / (1.f + expf(-z)) : -2.f;
  }
  int* lds_ids = reinterpret_cast<int*>(red);        // (a launch of one workgroup groups from here)
  __syncthreads();
  const int r = tid >> 5, q = tid & 31, row = r0 + r;  // 32 lanes per row: the choices stay inside a wave
  for (int k = 0; k < p.top; ++k) {
    float best = -3.f;
    int at = 0;
    for (int e = q; e < p.E; e += 32) {
      const float v = sc[r * (Ep + 1) + e];
      if (v > best) {
        best = v;
        at = e;
      }
    }
#pragma unroll
    for (int o = 16; o > 0; o >>= 1) {
      const float bo = __shfl_xor(best, o, 32);
      const int ao = __shfl_xor(at, o, 32);
      if (bo > best || (bo == best && ao < at)) {
        best = bo;
        at = ao;
      }
    }
    if (q == 0 && r < nr) {
      sc[r * (Ep + 1) + at] = -1.f;                  // (taken; scores are positive)
      p.wts[row * p.top + k] = live ? best : 0.f;
      lds_ids[r * p.top + k] = live ? at : -1;
      __hip_atomic_store(p.ids + row * p.top + k, live ? at : -1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  __syncthreads();
  if (gridDim.x == 1) {
    group_pairs(p, [&](int i) { return lds_ids[i]; });
    return;
  }
  // ---- the last workgroup groups the pairs
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (tid == 0) {
    const int t = __hip_atomic_fetch_add(p.ticket, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    s_last = t == (int)gridDim.x - 1;
    if (s_last) __hip_atomic_store(p.ticket, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  __syncthreads();
  if (!s_last) return;
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
  group_pairs(p, [&](int i) { return __hip_atomic_load(p.ids + i, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); });
}

// ------------------------------------------------------------------------------------------ small tiles (16 NP pairs)
// A workgroup per (tile, NU x 16 features | columns); its 4 waves split K, the sums meet in LDS.
template <class T, bool DOWN, int NP, int NU>
__global__ __launch_bounds__(256) void moe_small_kernel(MoeGemmParams p) {
  using M = MM<T>;
  constexpr int NA = DOWN ? 1 : 2;                   // 16-row tiles of the matrix per unit
  __shared__ float red[4][NP][NU][NA][64][4];
  const int tile = blockIdx.y;
  if (tile >= p.tiles[0]) return;
  const int e = p.tiles[1 + 3 * tile], place = p.tiles[2 + 3 * tile], n = p.tiles[3 + 3 * tile];
  const int lane = lane_id(), w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), rl = lane & 15, g = lane >> 4;
  const int KG = p.K / (16 * M::EPL), units = p.N / (16 * NA), unit0 = blockIdx.x * NU;
  const T* x[NP];
#pragma unroll
  for (int t = 0; t < NP; ++t) {
    const int src = place + min(16 * t + rl, n - 1);
    x[t] = reinterpret_cast<const T*>(p.x) + (size_t)(DOWN ? src : p.order[src] / p.top) * p.ldx + 4 * M::EPL * g;
  }
  const uint4* wp[NU];                               // (a unit past the matrix repeats its last one)
#pragma unroll
  for (int u = 0; u < NU; ++u)
    wp[u] = reinterpret_cast<const uint4*>(reinterpret_cast<const T*>(p.w) + e * p.w_expert) + (size_t)min(unit0 + u, units - 1) * NA * KG * 256;
  f32x4 acc[NP][NU][NA] = {};
  for (int kg = w; kg < KG; kg += 4) {
    uint4 f[NU][NA][4], a[NP][4];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
#pragma unroll
      for (int u = 0; u < NU; ++u)
#pragma unroll
        for (int j = 0; j < NA; ++j) f[u][j][s] = (wp[u] + ((size_t)j * KG + kg) * 256 + s * 64)[(unsigned)lane];
#pragma unroll
      for (int t = 0; t < NP; ++t) a[t][s] = *reinterpret_cast<const uint4*>(x[t] + kg * 16 * M::EPL + s * M::EPL);
    }
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int t = 0; t < NP; ++t)
#pragma unroll
        for (int u = 0; u < NU; ++u)
#pragma unroll
          for (int j = 0; j < NA; ++j) acc[t][u][j] = M::mma(a[t][s], f[u][j][s], acc[t][u][j]);
  }
#pragma unroll
  for (int t = 0; t < NP; ++t)
#pragma unroll
    for (int u = 0; u < NU; ++u)
#pragma unroll
      for (int j = 0; j < NA; ++j) *reinterpret_cast<f32x4*>(red[w][t][u][j][lane]) = acc[t][u][j];
  __syncthreads();
  // thread (lane, i = wave): pairs 16 t + 4 g + i, column rl
  T* y = reinterpret_cast<T*>(p.y);
#pragma unroll
  for (int t = 0; t < NP; ++t) {
    const int q = 16 * t + 4 * g + w;
    if (q >= n) continue;
    const int pair = p.order[place + q];
    const float score = DOWN ? 1.f : p.wts[pair];
    T* yr = y + (size_t)(DOWN ? pair : place + q) * p.ldy + unit0 * 16 + rl;
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      if (unit0 + u >= units) continue;
      float v[NA];
#pragma unroll
      for (int j = 0; j < NA; ++j)
        v[j] = (red[0][t][u][j][lane][w] + red[1][t][u][j][lane][w]) + (red[2][t][u][j][lane][w] + red[3][t][u][j][lane][w]);
      if constexpr (DOWN) stv(yr + u * 16, v[0]);
      else stv(yr + u * 16, silu(score * v[0]) * (score * v[1]));
    }
  }
}

// (units: as many matrix tiles per row of x read, gate / up or down)
template <class T, int NP>
void launch_small(const MoeGemmParams& p, hipStream_t st) {
  constexpr int NG = NP, ND = NP == 1 ? 1 : 2 * NP;
  const int units = p.N / (p.down ? 16 : 32), nu = p.down ? ND : NG;
  const dim3 grid((units + nu - 1) / nu, p.max_tiles), block(256);
  if (p.down) hipLaunchKernelGGL((moe_small_kernel<T, true, NP, ND>), grid, block, 0, st, p);
  else hipLaunchKernelGGL((moe_small_kernel<T, false, NP, NG>), grid, block, 0, st, p);
}

}  // namespace

extern "C" int vwa_moe_route(const MoeRouteParams* p, hipStream_t st) {
  if (p->rows < 1 || p->E < 1 || p->E > kMaxExperts || p->top < 1 || p->top > p->E || p->K % 32 || p->ldh % 8 || p->tile < 1 ||
      !p->wts || !p->ids || !p->tiles || !p->order || !p->ticket)
    return -1;
  // (every expert's last tile may be partly filled)
  const int64_t P = (int64_t)p->rows * p->top;
  if (p->max_tiles < (P < p->E ? P : p->E) + P / p->tile) return -2;
  const int Ep = (p->E + 15) / 16 * 16;
  const size_t lds = (size_t)kRouteWaves * Ep * 16 * 4 + 16 * (Ep + 1) * 4;
  if (lds > kMaxLds) return -10;
  const dim3 grid((p->rows + 15) / 16), block(kRouteThreads);
  if (p->f32) hipLaunchKernelGGL((moe_route_kernel<float>), grid, block, lds, st, *p);
  else hipLaunchKernelGGL((moe_route_kernel<u16>), grid, block, lds, st, *p);
  return (int)hipGetLastError();
}

extern "C" int vwa_moe_gemm(const MoeGemmParams* p, hipStream_t st) {
  if (p->max_tiles < 1 || p->N % (p->down ? 16 : 32) || p->K % 128 || p->ldx % 8 || (p->tile != 16 && p->tile != 32 && p->tile != 128 && p->tile != 256) || !p->tiles || !p->order ||
      (!p->down && !p->wts))
    return -1;
  if ((reinterpret_cast<uintptr_t>(p->x) | reinterpret_cast<uintptr_t>(p->w)) & 15) return -2;
  if (p->tile > 32) {
    if (p->f32) return -3;
    GemmParams q{};
    q.X = reinterpret_cast<const uint16_t*>(p->x);
    q.ldx = p->ldx;
    q.W = reinterpret_cast<const uint16_t*>(p->w);
    q.w_tiled = 1;
    q.M = p->x_rows;
    q.N = p->N;
    q.K = p->K;
    q.Y = p->y;
    q.ldy = p->ldy;
    q.rstd = p->down ? nullptr : p->wts;
    q.g_tiles = p->tiles;
    q.g_order = p->order;
    q.g_max = p->max_tiles;
    q.g_tile = p->tile;
    q.g_top = p->top;
    q.g_down = p->down;
    q.g_wstride = p->w_expert;
    return vwa_gemm_grouped(p->down ? 0 : 2, &q, st);
  }
  if (p->f32) p->tile == 16 ? launch_small<float, 1>(*p, st) : launch_small<float, 2>(*p, st);
  else p->tile == 16 ? launch_small<u16, 1>(*p, st) : launch_small<u16, 2>(*p, st);
  return (int)hipGetLastError();
}
