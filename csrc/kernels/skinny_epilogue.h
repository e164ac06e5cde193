// Epilogue and load helpers of the skinny decode GEMMs, shared by the streaming kernels
// (skinny_stream.hip) and the chained decode layer (chain.hip).
#pragma once
#include "common.h"
#include "vwa_kernels.h"

using namespace vwa;

namespace {

enum Epi { EPI_STORE = 0, EPI_RESID = 1, EPI_SWIGLU = 2, EPI_GELU = 3, EPI_QKV = 4, EPI_SPLIT = 5 };

constexpr unsigned kOOB = 0xFFFFFFF0u;

VWA_DEVICE uint4 bload(__amdgpu_buffer_rsrc_t r, unsigned off) {
  u32x4 v = __builtin_amdgcn_raw_buffer_load_b128(r, (int)off, 0, 0);
  return make_uint4(v.x, v.y, v.z, v.w);
}
// weight-stream load with cache policy AUX (gfx950 buffer aux bits: 1 sc0, 2 nt, 16 sc1): decode
// weights are read once per step by one CU, so nt (2) keeps them from displacing L2 lines
template <int AUX>
VWA_DEVICE uint4 bload_w(__amdgpu_buffer_rsrc_t r, unsigned off) {
  u32x4 v = __builtin_amdgcn_raw_buffer_load_b128(r, (int)off, 0, AUX);
  return make_uint4(v.x, v.y, v.z, v.w);
}
// the same with the constant part of the offset in soffset (a scalar): one VGPR offset per 4
// loads instead of one per load.  Past-the-end items use voff = kOOB2 (>= 2 GB, above every
// weight's num_records even with soffset added)
constexpr unsigned kOOB2 = 0x80000000u;
template <int AUX>
VWA_DEVICE uint4 bload_w_so(__amdgpu_buffer_rsrc_t r, unsigned voff, int soff) {
  u32x4 v = __builtin_amdgcn_raw_buffer_load_b128(r, (int)voff, soff, AUX);
  return make_uint4(v.x, v.y, v.z, v.w);
}

// Epilogue operands that do not depend on the GEMM (residual tile, fp8 column scales, QKV row
// positions / KV slots / rotary factors) are loaded for the workgroup's FIRST tile at kernel
// start, so they are not one more dependent memory round trip after the reduction.  Thread o
// owns output o of the tile (M*16*NT <= threads for every shape the launcher accepts).
struct EpiPre {
  float r = 0.f, cs0 = 1.f, cs1 = 1.f, rc = 1.f, rsn = 0.f;
  int64_t slot = -1;
};

// In-launch hand-off accessors (chain kernel): agent-scope relaxed atomics compile to sc1 loads /
// stores, which bypass the non-coherent per-XCD L2 state another workgroup could have left.
template <bool SC1>
VWA_DEVICE u16 ld_u16(const u16* p) {
  if constexpr (SC1) return __hip_atomic_load(gp(p), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  else return gld(p);
}
template <bool SC1>
VWA_DEVICE void st_u16(u16* p, u16 v) {
  if constexpr (SC1) __hip_atomic_store(gp(p), v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  else *gp(p) = v;
}
template <bool SC1>
VWA_DEVICE void st_f32(float* p, float v) {
  if constexpr (SC1) __hip_atomic_store(gp(p), v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  else *gp(p) = v;
}

template <int EPI, int NT, bool SC1 = false>
VWA_DEVICE void epi_values(const SkinnyParams& p, int tile, int o, EpiPre& e) {
  const int n0 = tile * 16 * NT;
  if constexpr (EPI == EPI_SWIGLU || EPI == EPI_QKV) {
    if (o >= p.M * 16) return;
    const int m = o >> 4, q = o & 15;
    if (p.w_scale) {
      e.cs0 = gld(p.w_scale + n0 + q);
      e.cs1 = gld(p.w_scale + n0 + (EPI == EPI_SWIGLU ? 16 + q : (q ^ 8)));
    }
    if constexpr (EPI == EPI_QKV) {
      const int hd = p.head_dim, half = hd >> 1, t = (n0 % hd) >> 4;
      e.slot = gld(p.slots + m);
      if (p.use_rope) {
        const int di = (q < 8) ? (8 * t + q) : (8 * t + q - 8);
        const int pos = gld(p.positions + m);
        e.rc = gld(p.rope + ((size_t)pos * half + di) * 2 + 0);
        e.rsn = gld(p.rope + ((size_t)pos * half + di) * 2 + 1);
      }
    }
  } else {
    if (o >= p.M * 16 * NT) return;
    const int m = o / (16 * NT), nn = o % (16 * NT);
    if (p.w_scale) e.cs0 = gld(p.w_scale + n0 + nn);
    if constexpr (EPI == EPI_RESID) {
      if (!SC1 && p.y_f32 == 2) e.r = gld(reinterpret_cast<const float*>(p.R) + (size_t)m * p.ldr + n0 + nn);
      else e.r = p.R ? bf2f(ld_u16<SC1>(p.R + (size_t)m * p.ldr + n0 + nn)) : 0.f;
    }
  }
}

// Cross-wave reduction of one column tile + fused epilogue.  rs[m]: per-row scale (fused RMSNorm
// / LayerNorm rstd and, on the fp8 path, the activation quantisation scale); mus[m] (folded
// LayerNorm only, else null): row mean, removed as mean * ln_c[n]; column scales (fp8) come
// with the epilogue operands (`pre` when this is the workgroup's first tile).
// MT: 16-row MFMA row fragments per tile (M <= 16 MT; MT > 1 only in the streaming kernel's
// many-row form, skinny_stream_kernel); red = [KS][NT][MT][4][64] partial sums.
template <int EPI, int NT, int KS, bool SC1 = false, int MT = 1>
VWA_DEVICE void tile_epilogue(const SkinnyParams& p, float* red, const float* rs, const float* mus, int tile,
                              f32x4 (&acc)[NT * MT], int w, int lane, const EpiPre& pre, bool first,
                              const float* partner = nullptr) {
  const int M = p.M;
  const int n0 = tile * 16 * NT;
#pragma unroll
  for (int nt = 0; nt < NT; ++nt)
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
      for (int i = 0; i < 4; ++i) red[(((w * NT + nt) * MT + mt) * 4 + i) * 64 + lane] = acc[nt * MT + mt][i];
  lds_sync();
  auto red_at = [&](int m, int nn) -> float {
    const int nt = nn >> 4, q = nn & 15, mt = MT > 1 ? m >> 4 : 0, mm = m & 15;
    const int ln = q + 16 * (mm >> 2), i = mm & 3;
    float s = 0.f;
#pragma unroll
    for (int ww = 0; ww < KS; ++ww) s += red[(((ww * NT + nt) * MT + mt) * 4 + i) * 64 + ln];
    // split tile (chain kernel): the other workgroup's partial sums, published with sc1 stores
    if (partner) s += __hip_atomic_load(gp(partner + m * 16 * NT + nn), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    return s;
  };
  auto operands = [&](int o) {
    if (first && o == VWA_TX) return pre;
    EpiPre e;
    epi_values<EPI, NT, SC1>(p, tile, o, e);
    return e;
  };
  if constexpr (EPI == EPI_SWIGLU) {
    for (int o = VWA_TX; o < M * 16; o += KS * 64) {
      const int m = o >> 4, q = o & 15;
      const EpiPre e = operands(o);
      const float sc = rs[m];
      float gv = red_at(m, q) * sc * e.cs0, uv = red_at(m, 16 + q) * sc * e.cs1;
      if (p.bias) {
        gv += bf2f(gld(p.bias + n0 + q));
        uv += bf2f(gld(p.bias + n0 + 16 + q));
      }
      st_u16<SC1>(reinterpret_cast<u16*>(p.Y) + (size_t)m * p.ldy + tile * 16 + q, f2bf(silu(gv) * uv));
    }
  } else if constexpr (EPI == EPI_QKV) {
    const int hd = p.head_dim, half = hd >> 1;
    const int head = n0 / hd;
    const int t = (n0 % hd) >> 4;
    const bool is_v = head >= p.n_q_heads + p.n_kv_heads;
    for (int o = VWA_TX; o < M * 16; o += KS * 64) {
      const int m = o >> 4, q = o & 15;
      const EpiPre e = operands(o);
      const float sc = rs[m];
      float v = red_at(m, q), pv = red_at(m, q ^ 8);
      if (mus) {
        v -= mus[m] * gld(p.ln_c + n0 + q);
        pv -= mus[m] * gld(p.ln_c + n0 + (q ^ 8));
      }
      v *= sc * e.cs0;
      pv *= sc * e.cs1;
      if (p.bias) {
        v += bf2f(gld(p.bias + n0 + q));
        pv += bf2f(gld(p.bias + n0 + (q ^ 8)));
      }
      const int d = (q < 8) ? (8 * t + q) : (half + 8 * t + q - 8);
      if (p.use_rope && !is_v) v = (q < 8) ? (v * e.rc - pv * e.rsn) : (v * e.rc + pv * e.rsn);
      const u16 out = f2bf(v);
      if (head < p.n_q_heads) {
        st_u16<SC1>(p.q_out + (size_t)m * p.ldq + head * hd + d, out);
      } else {
        const int64_t slot = e.slot;
        if (slot >= 0) {
          const int64_t blk = slot / p.block_size, off = slot % p.block_size;
          const int kvh = is_v ? head - p.n_q_heads - p.n_kv_heads : head - p.n_q_heads;
          const int64_t idx = blk * p.cache_stride_block + kvh * p.cache_stride_head + off * p.cache_stride_tok + d;
          st_u16<SC1>((is_v ? p.v_cache : p.k_cache) + idx, out);
        }
      }
    }
  } else {
    for (int o = VWA_TX; o < M * 16 * NT; o += KS * 64) {
      const int m = o / (16 * NT), nn = o % (16 * NT);
      const int n = n0 + nn;
      const EpiPre e = operands(o);
      float v = red_at(m, nn);
      if (mus) v -= mus[m] * gld(p.ln_c + n);
      v *= rs[m] * e.cs0;
      if (p.bias) v += bf2f(gld(p.bias + n));
      if constexpr (EPI == EPI_GELU) v = gelu_erf(v);
      if constexpr (EPI == EPI_RESID) v += e.r;
      if constexpr (EPI == EPI_SPLIT) {
        if (n0 >= p.n_q_heads) {  // (the split is a multiple of the 16-column tile)
          v = fmaxf(v, 0.f);
          st_u16<SC1>(p.q_out + (size_t)m * p.ldq + n - p.n_q_heads, f2bf(v * v));
          continue;
        }
      }
      if (p.y_f32) st_f32<SC1>(reinterpret_cast<float*>(p.Y) + (size_t)m * p.ldy + n, v);
      else st_u16<SC1>(reinterpret_cast<u16*>(p.Y) + (size_t)m * p.ldy + n, f2bf(v));
    }
  }
  lds_sync();
#pragma unroll
  for (int k = 0; k < NT * MT; ++k) acc[k] = f32x4{0.f, 0.f, 0.f, 0.f};
}

}  // namespace
