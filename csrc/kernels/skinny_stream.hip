// Streaming skinny GEMM (decode path, M <= 16 typically) -- persistent, software-pipelined.
//
// Same math and epilogues as skinny_gemm.hip, restructured after rocprof showed the one-tile-
// per-workgroup kernel streaming weights at only ~3.1-3.4 TB/s: every workgroup paid launch +
// prologue + LDS reduction + epilogue around a single round trip of weight loads, leaving the
// CU's memory pipe idle between workgroups.  Here:
//
//  * X (the activation rows, <= ~140 KB) is staged in LDS once per workgroup and read back with
//    ds_read_b128 -- no activation loads in the weight stream, no X registers;
//  * the fused-RMSNorm row scales are computed once from that LDS copy;
//  * each workgroup is persistent over column tiles (tile = blockIdx.x + i*gridDim.x); its KS
//    waves split K, and every wave walks a flat list of (tile, k-batch) items;
//  * weight loads are raw buffer loads (SRD with num_records = N*K*2): the next item's 16 x
//    dwordx4 per lane are issued BEFORE the current item's MFMAs (two named register sets,
//    static indices -> counted vmcnt), and past-the-end items/groups use an out-of-range offset
//    that the hardware answers with zeros and no memory traffic, so the pipeline has no
//    data-dependent load predicates;
//  * the cross-wave reduction + fused epilogue of tile t runs while tile t+1's loads are in flight.
//
// XG variant (X does not fit in LDS: e.g. the down projection, K = 14336, with more than 5 rows):
// the activation fragments are streamed from global memory alongside the weights (X is a few
// hundred KB and stays L2-resident, so the extra loads hit L2, not HBM), with the same
// two-register-set pipeline; only the reduction scratch lives in LDS.
#include "skinny_epilogue.h"

namespace {

// MT: 16-row MFMA row fragments per weight fragment (only MT = 1 is instantiated since round 5: the
// 17..64-row form measured slower than the tiled GEMM and was removed).
template <int EPI, int NT, int KS, bool XG, int MT = 1>
__global__ __launch_bounds__(KS * 64) void skinny_stream_kernel(SkinnyParams p, int nb, int xstride, int xskew) {
  // k-groups (128 wide) per item; MT > 1: one (the X fragments of MT row tiles share the
  // register budget of the item's weights)
  constexpr int U = MT > 1 ? 1 : XG ? 2 : 4 / NT;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int M = p.M, K = p.K, N = p.N;
  u16* xs = reinterpret_cast<u16*>(smem);
  // LDS-staged X: row m at m * xstride + (m / 4) * xskew elements.  xstride = K + 8 puts row m+1
  // one 16-B bank slot after row m; the extra 64-B skew every 4 rows (xskew 32) makes each
  // ds_read_b128 lane group ({0-3,12-15,20-27}, ...: rows nl, k-quarters g) hit 16 distinct slots
  // -- without it lanes (nl, g) and (nl + 4, g - 1)... share slots, a 2-way conflict on every read.
  const int xbytes = XG ? 0 : ((M * xstride * 2) + 4 * xskew * 2 + 15) & ~15;
  float* red = reinterpret_cast<float*>(smem + xbytes);  // [KS][NT][MT][4][64]
  auto xrow = [&](int m) { return m * xstride + (m >> 2) * xskew; };
  float* rs = red + KS * NT * MT * 4 * 64;                // [16 MT] row scales (1/rms, LayerNorm rstd)
  float* mu = rs + 16 * MT;                               // [16 MT] row means (folded LayerNorm)
  const float* mus = (p.fuse_rms == 2) ? mu : nullptr;
  const int lane = VWA_TX & 63, w = VWA_TX >> 6;
  const int nl = lane & 15, g = lane >> 4;

  EpiPre pre;
  epi_values<EPI, NT>(p, blockIdx.x, VWA_TX, pre);  // first tile's epilogue operands, early
  const int G = K / 128;
  const int gb = (G * w) / KS, ge = (G * (w + 1)) / KS;
  const __amdgpu_buffer_rsrc_t rw =
      __builtin_amdgcn_make_buffer_rsrc(const_cast<u16*>(p.W), (short)0, (int)((size_t)N * K * 2), 0x00020000);
  // X fragments (XG): lane (row nl, k-quarter g); rows >= M read the zero OOB answer
  const __amdgpu_buffer_rsrc_t rx =
      __builtin_amdgcn_make_buffer_rsrc(const_cast<u16*>(p.X), (short)0, (int)((size_t)M * p.ldx * 2), 0x00020000);
  const int ntiles = N / (16 * NT);
  const int my_tiles = (ntiles - (int)blockIdx.x + (int)gridDim.x - 1) / (int)gridDim.x;
  // grammar-masked LM head (p.col_mask; the launcher keeps it only for NT 1, EPI store, LDS-staged
  // X and <= 64 tiles per workgroup): this workgroup's tiles that hold an admissible token of some
  // row, compacted into lanes (lane k: the k-th live tile).  Measured on the intent grammar: 42 %
  // of the LM head's tiles live per decode step on average, 10 % at the median.
  const bool masked = NT == 1 && !XG && p.col_mask != nullptr;
  int n_live = my_tiles, live_tile = 0;
  if (masked) {
    const int tl = (int)blockIdx.x + lane * (int)gridDim.x;
    unsigned bits = 0;
    if (lane < my_tiles)
      for (int r = 0; r < p.col_mask_rows; ++r) bits |= p.col_mask[(size_t)r * p.col_mask_ld + (tl >> 1)];
    bits = (tl & 1) ? (bits >> 16) : (bits & 0xFFFFu);
    const unsigned long long live = __ballot(lane < my_tiles && bits != 0u);
    n_live = __popcll(live);
    const int rank = __popcll(live & ((1ull << lane) - 1ull));
    const int dst = ((live >> lane) & 1ull) ? rank : n_live + (lane - rank);  // a permutation of the lanes
    live_tile = __builtin_amdgcn_ds_permute(dst * 4, tl);
  }
  const int n_items = n_live * nb;
  auto tile_of = [&](int it) { return masked ? __shfl(live_tile, it / nb, 64) : (int)blockIdx.x + (it / nb) * (int)gridDim.x; };

  auto load_x = [&](uint4 (&xr)[MT][U][4], int it) {
    const int b = it % nb;
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int kg = gb + b * U + u, row = 16 * mt + nl;
        const bool ok = (it < n_items) && (kg < ge) && (row < M);
        const unsigned base = ((unsigned)row * (unsigned)p.ldx + (unsigned)(kg * 128 + 32 * g)) * 2u;
#pragma unroll
        for (int s = 0; s < 4; ++s) xr[mt][u][s] = bload(rx, ok ? base + 16u * s : kOOB);
      }
  };

  auto load_item = [&](uint4 (&wr)[NT][U][4], int it) {
    const int tile = tile_of(it);
    const int b = it % nb;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int kg = gb + b * U + u;
      const bool ok = (it < n_items) && (kg < ge);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        if (p.w_tiled) {  // pre-tiled: 1 KB contiguous per load instruction
          const unsigned T = (unsigned)(tile * NT + nt);
          const unsigned base = ((T * (unsigned)G + (unsigned)kg) * 4u) * 1024u + (unsigned)lane * 16u;
#pragma unroll
          for (int s = 0; s < 4; ++s) wr[nt][u][s] = bload(rw, ok ? base + 1024u * s : kOOB);
        } else {
          const unsigned row = (unsigned)(tile * 16 * NT + nt * 16 + nl);
          const unsigned base = (row * (unsigned)K + (unsigned)(kg * 128 + 32 * g)) * 2u;
#pragma unroll
          for (int s = 0; s < 4; ++s) wr[nt][u][s] = bload(rw, ok ? base + 16u * s : kOOB);
        }
      }
    }
  };

  f32x4 acc[NT * MT];
#pragma unroll
  for (int k = 0; k < NT * MT; ++k) acc[k] = f32x4{0.f, 0.f, 0.f, 0.f};

  auto compute_item = [&](const uint4 (&wr)[NT][U][4], const uint4 (&xr)[MT][U][4], int it) {
    const int b = it % nb;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int kg = gb + b * U + u;
      if (kg >= ge) break;  // wave-uniform
#pragma unroll
      for (int s = 0; s < 4; ++s) {
#pragma unroll
        for (int mt = 0; mt < MT; ++mt) {
          uint4 a = make_uint4(0, 0, 0, 0);
          if constexpr (XG) a = xr[mt][u][s];
          else if (16 * mt + nl < M)
            a = *reinterpret_cast<const uint4*>(xs + xrow(16 * mt + nl) + kg * 128 + 32 * g + 8 * s);
#pragma unroll
          for (int nt = 0; nt < NT; ++nt)
            acc[nt * MT + mt] = mfma16(as_bf16x8(a), as_bf16x8(wr[nt][u][s]), acc[nt * MT + mt]);
        }
      }
    }
  };

  auto finish_tile = [&](int it) {
    tile_epilogue<EPI, NT, KS, false, MT>(p, red, rs, mus, tile_of(it), acc, w, lane, pre, !masked && it < nb);
  };

  uint4 A[NT][U][4], B[NT][U][4];
  uint4 XA[MT][U][4], XB[MT][U][4];  // XG only (dead otherwise)
  // w_first: issue the first weight item before staging X (its round trip then overlaps the X
  // staging + fused-RMSNorm statistics); otherwise stage X first (the X round trip is short).
  if (p.w_first) {
    load_item(A, 0);
    if constexpr (XG) load_x(XA, 0);
  }
  // ---- stage X rows into LDS
  const int k8 = K / 8;
  if constexpr (!XG) {
    for (int c = VWA_TX; c < M * k8; c += KS * 64) {
      const int m = c / k8, kk = c % k8;
      *reinterpret_cast<uint4*>(xs + xrow(m) + kk * 8) =
          *reinterpret_cast<const uint4*>(p.X + (size_t)m * p.ldx + kk * 8);
    }
  }
  lds_sync();
  for (int m = w; m < 16 * MT; m += KS) {
    float sc = 1.f, mean = 0.f;
    if (p.fuse_rms && m < M) {
      float s = 0.f, s1 = 0.f;
      for (int kk = lane; kk < k8; kk += 64) {
        float f[8];
        unpack8(XG ? *reinterpret_cast<const uint4*>(p.X + (size_t)m * p.ldx + kk * 8)
                   : *reinterpret_cast<const uint4*>(xs + xrow(m) + kk * 8), f);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          s += f[j] * f[j];
          s1 += f[j];
        }
      }
      s = wave_sum(s);
      if (p.fuse_rms == 2) {  // LayerNorm: rstd from E[x^2] - mean^2
        mean = wave_sum(s1) / (float)K;
        sc = rsqrtf(fmaxf(s / (float)K - mean * mean, 0.f) + p.eps);
      } else {
        sc = rsqrtf(s / (float)K + p.eps);
      }
    }
    if (lane == 0) {
      rs[m] = sc;
      mu[m] = mean;
    }
  }
  lds_sync();

  if (!p.w_first) {
    load_item(A, 0);
    if constexpr (XG) load_x(XA, 0);
  }
  // the next item into a register set is issued right after that set's compute, BEFORE the tile
  // epilogue, so two items stay in flight through every epilogue
  load_item(B, 1);
  if constexpr (XG) load_x(XB, 1);
  for (int it = 0; it < n_items; it += 2) {
    compute_item(A, XA, it);
    load_item(A, it + 2);
    if constexpr (XG) load_x(XA, it + 2);
    if (it % nb == nb - 1) finish_tile(it);
    if (it + 1 >= n_items) break;
    compute_item(B, XB, it + 1);
    load_item(B, it + 3);
    if constexpr (XG) load_x(XB, it + 3);
    if ((it + 1) % nb == nb - 1) finish_tile(it + 1);
  }
}

int g_x_skew = 32;  // LDS X row skew (elements per 4 rows; 0: none -- A/B knob, vwa_skinny_set_x_skew)

template <int EPI, int NT, int KS, bool XG, int MT = 1>
int launch_v(const SkinnyParams& p, hipStream_t st, int grid_cap, size_t lds, int xstride) {
  constexpr int U = MT > 1 ? 1 : XG ? 2 : 4 / NT;
  const int G = p.K / 128;
  const int per_wave = (G + KS - 1) / KS;
  const int nb = (per_wave + U - 1) / U;
  const int ntiles = p.N / (16 * NT);
  const int grid = ntiles < grid_cap ? ntiles : grid_cap;
  hipLaunchKernelGGL((skinny_stream_kernel<EPI, NT, KS, XG, MT>), dim3(grid), dim3(KS * 64), lds, st, p, nb, xstride,
                     XG ? 0 : g_x_skew);
  return 0;
}

template <int EPI, int NT, int KS>
int launch(const SkinnyParams& p0, hipStream_t st, int grid_cap) {
  SkinnyParams p = p0;
  const int xstride = p.K + 8;
  // (round 4's 17..64-row form -- X streamed next to the weights, 2 / 4 row fragments per weight
  // fragment -- measured slower than the tiled GEMM for whole decode steps and was removed in round
  // 5: more than 16 rows are the tiled GEMM's, gemm.hip)
  if (p.M > 16) return -10;
  const size_t xbytes = ((size_t)p.M * xstride * 2 + 4 * g_x_skew * 2 + 15) & ~(size_t)15;
  const size_t red = (size_t)(KS * NT * 4 * 64 + 32) * sizeof(float);  // + row scales + row means
  // X rows staged in LDS when they fit next to the reduction scratch; otherwise (the down
  // projection's 14336-wide rows at more than ~5 rows) streamed from L2 with the weights (XG)
  const bool lds_x = xbytes + red <= 160 * 1024;
  if (p.col_mask) {  // the masked tile list: NT 1, EPI store, LDS-staged X, <= 64 tiles per workgroup
    const int ntiles = p.N / (16 * NT), grid = ntiles < grid_cap ? ntiles : grid_cap;
    if (EPI != EPI_STORE || NT != 1 || !lds_x || (ntiles + grid - 1) / grid > 64 || p.col_mask_rows < 1)
      p.col_mask = nullptr;
  }
  if (lds_x) return launch_v<EPI, NT, KS, false>(p, st, grid_cap, xbytes + red, xstride);
  if ((size_t)p.M * p.ldx * 2 >= 0x7FFFFFF0ull) return -10;
  return launch_v<EPI, NT, KS, true>(p, st, grid_cap, red, xstride);
}


// ------------------------------------------------------------------------------------------
// W8A8 variant (VWA_DTYPE=fp8): W is OCP e4m3 [N, K] bytes with per-row scales, X rows are
// quantised to e4m3 once per workgroup while staging into LDS (per-row dynamic scale
// amax/448), the inner product runs on the fp8 MFMA (16x16x32, 8 bytes per lane per operand),
// and both scales are applied in the epilogue.  Weight bytes per decode step are halved.
// ------------------------------------------------------------------------------------------
template <int EPI, int NT, int KS>
__global__ __launch_bounds__(KS * 64) void skinny_fp8_kernel(SkinnyParams p, int nb, int xstride) {
  constexpr int U = 8 / NT;  // k-groups (128 wide) per item: 2 x b128 weight loads per k-group
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int M = p.M, K = p.K, N = p.N;
  uint8_t* xs = reinterpret_cast<uint8_t*>(smem);
  const int xbytes = ((M * xstride) + 15) & ~15;
  float* red = reinterpret_cast<float*>(smem + xbytes);  // [KS][NT][4][64]
  float* rs = red + KS * NT * 4 * 64;                     // [16] row scale (rms * x-quant scale)
  float* inv = rs + 16;                                    // [16] 1 / x-quant scale
  const int lane = VWA_TX & 63, w = VWA_TX >> 6;
  const int nl = lane & 15, g = lane >> 4;
  const int k8 = K / 8;

  EpiPre pre;
  epi_values<EPI, NT>(p, blockIdx.x, VWA_TX, pre);  // first tile's epilogue operands, early
  // ---- per-row statistics (sum of squares for the fused RMSNorm, amax for the fp8 scale)
  for (int m = w; m < 16; m += KS) {
    float sc = 1.f, iv = 1.f;
    if (m < M) {
      float ss = 0.f, am = 0.f;
      for (int kk = lane; kk < k8; kk += 64) {
        float f[8];
        unpack8(*reinterpret_cast<const uint4*>(p.X + (size_t)m * p.ldx + kk * 8), f);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          ss += f[j] * f[j];
          am = fmaxf(am, fabsf(f[j]));
        }
      }
      ss = wave_sum(ss);
      am = wave_max(am);
      const float sx = am > 0.f ? am * (1.f / 448.f) : 1.f;
      iv = 1.f / sx;
      sc = (p.fuse_rms ? rsqrtf(ss / (float)K + p.eps) : 1.f) * sx;
    }
    if (lane == 0) {
      rs[m] = sc;
      inv[m] = iv;
    }
  }
  lds_sync();
  // ---- quantise X rows into LDS (e4m3, 8 values -> 8 bytes)
  for (int c = VWA_TX; c < M * k8; c += KS * 64) {
    const int m = c / k8, kk = c % k8;
    float f[8];
    unpack8(*reinterpret_cast<const uint4*>(p.X + (size_t)m * p.ldx + kk * 8), f);
    const float iv = inv[m];
    uint2 q;
    q.x = cvt_pk_fp8(f[0] * iv, f[1] * iv) | (cvt_pk_fp8(f[2] * iv, f[3] * iv) << 16);
    q.y = cvt_pk_fp8(f[4] * iv, f[5] * iv) | (cvt_pk_fp8(f[6] * iv, f[7] * iv) << 16);
    *reinterpret_cast<uint2*>(xs + m * xstride + kk * 8) = q;
  }
  lds_sync();

  const int G = K / 128;
  const int gb = (G * w) / KS, ge = (G * (w + 1)) / KS;
  const __amdgpu_buffer_rsrc_t rw =
      __builtin_amdgcn_make_buffer_rsrc(const_cast<u16*>(p.W), (short)0, (int)((size_t)N * K), 0x00020000);
  const int ntiles = N / (16 * NT);
  const int my_tiles = (ntiles - (int)blockIdx.x + (int)gridDim.x - 1) / (int)gridDim.x;
  const int n_items = my_tiles * nb;

  auto load_item = [&](uint4 (&wr)[NT][U][2], int it) {
    const int tile = blockIdx.x + (it / nb) * gridDim.x;
    const int b = it % nb;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int kg = gb + b * U + u;
      const bool ok = (it < n_items) && (kg < ge);
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        if (p.w_tiled) {
          // fp8 tiled layout (ops.tile_weight_fp8): the (16-row tile, k-group) block is 2 KB
          // [s][lane][16 B] -- each load instruction reads 1 KB contiguous, lane (nl, g) gets
          // W[row][128 kg + 32 g + 16 s .. + 16), the same bytes as the row-major addressing below
          const unsigned T = (unsigned)(tile * NT + nt);
          const unsigned base = (T * (unsigned)G + (unsigned)kg) * 2048u + (unsigned)lane * 16u;
#pragma unroll
          for (int s = 0; s < 2; ++s) wr[nt][u][s] = bload(rw, ok ? base + 1024u * s : kOOB);
        } else {
          const unsigned row = (unsigned)(tile * 16 * NT + nt * 16 + nl);
          const unsigned base = row * (unsigned)K + (unsigned)(kg * 128 + 32 * g);
#pragma unroll
          for (int s = 0; s < 2; ++s) wr[nt][u][s] = bload(rw, ok ? base + 16u * s : kOOB);
        }
      }
    }
  };

  f32x4 acc[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) acc[nt] = f32x4{0.f, 0.f, 0.f, 0.f};

  auto compute_item = [&](const uint4 (&wr)[NT][U][2], int it) {
    const int b = it % nb;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int kg = gb + b * U + u;
      if (kg >= ge) break;  // wave-uniform
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        uint4 a = make_uint4(0, 0, 0, 0);
        if (nl < M) a = *reinterpret_cast<const uint4*>(xs + nl * xstride + kg * 128 + 32 * g + 16 * s);
        const long a0 = (long)(((unsigned long)a.y << 32) | a.x), a1 = (long)(((unsigned long)a.w << 32) | a.z);
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          const uint4 v = wr[nt][u][s];
          const long b0 = (long)(((unsigned long)v.y << 32) | v.x), b1 = (long)(((unsigned long)v.w << 32) | v.z);
          acc[nt] = mfma16_fp8(a0, b0, acc[nt]);
          acc[nt] = mfma16_fp8(a1, b1, acc[nt]);
        }
      }
    }
  };

  uint4 A[NT][U][2], B[NT][U][2];
  load_item(A, 0);
  for (int it = 0; it < n_items; it += 2) {
    load_item(B, it + 1);
    compute_item(A, it);
    if (it % nb == nb - 1)
      tile_epilogue<EPI, NT, KS>(p, red, rs, nullptr, blockIdx.x + (it / nb) * gridDim.x, acc, w, lane, pre, it < nb);
    if (it + 1 >= n_items) break;
    load_item(A, it + 2);
    compute_item(B, it + 1);
    if ((it + 1) % nb == nb - 1)
      tile_epilogue<EPI, NT, KS>(p, red, rs, nullptr, blockIdx.x + ((it + 1) / nb) * gridDim.x, acc, w, lane, pre,
                                 it + 1 < nb);
  }
}

template <int EPI, int NT, int KS>
int launch_fp8(const SkinnyParams& p, hipStream_t st, int grid_cap) {
  constexpr int U = 8 / NT;
  // skinny_fp8_kernel holds 16 rows (rs[16], one MFMA row fragment): more rows must go to the
  // tiled GEMM, never to silently wrong rows 16+
  if (p.M > 16) return -10;
  const int G = p.K / 128;
  const int per_wave = (G + KS - 1) / KS;
  const int nb = (per_wave + U - 1) / U;
  const int xstride = p.K + 16;
  const size_t xbytes = ((size_t)p.M * xstride + 15) & ~(size_t)15;
  const size_t lds = xbytes + (size_t)(KS * NT * 4 * 64 + 32) * sizeof(float);
  if (lds > 160 * 1024) return -10;
  const int ntiles = p.N / (16 * NT);
  const int grid = ntiles < grid_cap ? ntiles : grid_cap;
  hipLaunchKernelGGL((skinny_fp8_kernel<EPI, NT, KS>), dim3(grid), dim3(KS * 64), lds, st, p, nb, xstride);
  return 0;
}

}  // namespace

// (round 4's 32-column tiles for the plain epilogues measured slower at
// 8 / 16 rows, profiles/r4_skinny_nt2_rows.jsonl, and were removed in round 5)

// Returns -10 when this shape does not fit the streaming kernel (caller falls back).
template <int KS>
int dispatch_ks(int epi, const SkinnyParams& p, int grid_cap, hipStream_t st) {
  if (p.w_scale) {
    switch (epi) {
      case EPI_STORE: return launch_fp8<EPI_STORE, 1, KS>(p, st, grid_cap);
      case EPI_RESID: return launch_fp8<EPI_RESID, 1, KS>(p, st, grid_cap);
      case EPI_GELU: return launch_fp8<EPI_GELU, 1, KS>(p, st, grid_cap);
      case EPI_SWIGLU: return launch_fp8<EPI_SWIGLU, 2, KS>(p, st, grid_cap);
      case EPI_QKV: return launch_fp8<EPI_QKV, 1, KS>(p, st, grid_cap);
      default: return -3;
    }
  }
  switch (epi) {
    case EPI_STORE: return launch<EPI_STORE, 1, KS>(p, st, grid_cap);
    case EPI_RESID: return launch<EPI_RESID, 1, KS>(p, st, grid_cap);
    case EPI_GELU: return launch<EPI_GELU, 1, KS>(p, st, grid_cap);
    case EPI_SWIGLU: return launch<EPI_SWIGLU, 2, KS>(p, st, grid_cap);
    case EPI_QKV: return launch<EPI_QKV, 1, KS>(p, st, grid_cap);
    case EPI_SPLIT: return p.n_q_heads % 16 || !p.q_out ? -4 : launch<EPI_SPLIT, 1, KS>(p, st, grid_cap);
    default: return -3;
  }
}

// Returns -10 when this shape does not fit the streaming kernel (caller falls back).
// ks = waves per workgroup splitting K (4 or 8); grid_cap = max persistent workgroups.
extern "C" void vwa_skinny_set_x_skew(int skew) { g_x_skew = skew == 0 ? 0 : 32; }

extern "C" int vwa_skinny_stream(int epi, const SkinnyParams* p, int grid_cap, int ks, hipStream_t st) {
  if (p->M < 1 || p->M > 16 || p->K % 128 != 0) return -10;
  if ((size_t)p->N * p->K * (p->w_scale ? 1 : 2) >= 0x7FFFFFF0ull) return -10;
#ifdef VWA_ONLY_MULTI
  const int r = -10;
#else
  const int r = (ks == 4) ? dispatch_ks<4>(epi, *p, grid_cap, st) : dispatch_ks<8>(epi, *p, grid_cap, st);
#endif
  if (r) return r;
  return (int)hipGetLastError();
}
