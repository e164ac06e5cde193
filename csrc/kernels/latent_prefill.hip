// Latent attention of prompt-sized runs (bf16): the cached latents of a run's context are gathered, expanded to
// every head's keys and values by one GEMM, and a flash kernel walks them -- per (query, key, head) that is
// dim + rot + vd products instead of the latent form's 2 rank + rot.
//
//  latent_gather  : context rows of the runs -> [T][latent padded to the GEMM's k] and [T][rotated key part]
//  latent_prefill : 128 queries of a run and one head per workgroup, 4 query waves x 2 key splits, 32-key tiles
//
// A wave owns 32 queries: S^T = K.Q^T with v_mfma_f32_32x32x16_bf16, the K rows of a tile read in an order that
// leaves lane half h with keys 8h.. and 16 + 8h.. of its query -- the B operand of O^T += V^T.P^T as it is.
// V^T comes from the row-major LDS image with ds_read_b64_tr_b16.  Row strides (K: 16 bytes past a multiple of
// 64; V: 64 past a multiple of 128) keep both reads spread over the banks.  Splits take tiles s, s + 2, ..,
// double-buffered in LDS with the next tile's loads in registers, and merge at the end with the head's sink.
#include "mixer_kernels.h"
#include "mq_attention.h"
#include "stack_types.h"

using namespace vwa;

namespace {

constexpr int kPQ = 128, kPK = 32, kNS = 2;
constexpr float kRescale = 8.f;                      // the running maximum moves when a tile exceeds it by this (log2)
constexpr float kLog2e = 1.4426950408889634f;

typedef float f32x16 __attribute__((ext_vector_type(16)));
VWA_DEVICE f32x16 mfma32(const bf16x8& a, const bf16x8& b, const f32x16& c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}

__global__ __launch_bounds__(256) void latent_gather_kernel(LatentPrefillParams p) {
  const int seg = blockIdx.x / 4, r0 = (blockIdx.x & 3) * 16;
  const int seq = p.segs[3 * seg], key0 = p.segs[3 * seg + 1], ctx = p.segs[3 * seg + 2];
  const int cr = p.rank_p / 8, cp = p.kp / 8, per = cp + p.rot_p / 8, dk = p.rank_p + p.rot_p;
  const int lb = __builtin_ctz(p.block_size);
  for (int i = threadIdx.x; i < 16 * per; i += 256) {
    const int r = r0 + i / per, c = i % per, t = seg * 64 + r;
    const int key = min(key0 + r, ctx - 1);
    const int blk = p.block_table[(int64_t)seq * p.table_stride + (key >> lb)];
    const u16* src = reinterpret_cast<const u16*>(p.cache) + (int64_t)blk * p.c_sb + (int64_t)(key & (p.block_size - 1)) * dk;
    if (c < cp)
      *reinterpret_cast<uint4*>(p.lat + (size_t)t * p.kp + c * 8) = c < cr ? ld128(src + c * 8) : make_uint4(0, 0, 0, 0);
    else
      *reinterpret_cast<uint4*>(p.krot + (size_t)t * p.rot_p + (c - cp) * 8) = ld128(src + p.rank_p + (c - cp) * 8);
  }
}

VWA_DEVICE int k_stride(int dk) { return dk * 2 + 16; }
VWA_DEVICE int v_stride(int vd) { return vd * 2 + ((vd * 2) % 128 == 0 ? 64 : 0); }
size_t prefill_lds(int dk, int vd, int ndt) {
  const size_t tiles = (size_t)kNS * 2 * kPK * (dk * 2 + 16 + vd * 2 + 64);
  const size_t merge = (size_t)(kNS - 1) * 4 * 64 * (ndt * 16 + 2) * 4;
  return tiles > merge ? tiles : merge;
}

// NDS: 16-wide steps over the query / key dimensions, NDT: 32-column value tiles (at most; narrower heads
// multiply zero queries / drop columns)
template <int NDS, int NDT>
__global__ __launch_bounds__(256 * kNS) void latent_prefill_kernel(LatentPrefillParams p) {
  constexpr int LK = (NDS * 2 * kPK + 255) / 256, LV = (NDT * 4 * kPK + 255) / 256;   // 16-byte pieces per thread and tile
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int L = xcd_remap((int)blockIdx.x, p.n_tiles * p.H);
  const int h = L / p.n_tiles, qt = L % p.n_tiles;
  const int row0 = p.q_tiles[4 * qt], nq = p.q_tiles[4 * qt + 1], t0 = p.q_tiles[4 * qt + 2], pos0 = p.q_tiles[4 * qt + 3];
  const int lane = lane_id(), wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int w = wid & 3, split = wid >> 2, stid = threadIdx.x & 255;
  const int col = lane & 31, hf = lane >> 5;
  const int dk = p.dim_p + p.rot_p, vdk = p.vdk, nds = dk >> 4;
  const int ks = k_stride(dk), vs = v_stride(vdk), tile_b = kPK * (ks + vs);
  unsigned char* simg = smem + split * 2 * tile_b;   // this split's [stage][K, V]
  const int qi = w * 32 + col, qrow = row0 + min(qi, nq - 1), qpos = pos0 + qi, qw0 = pos0 + w * 32;
  const float sl2 = p.scale * kLog2e;
  const int Sk = pos0 + nq, nt = (Sk + kPK - 1) / kPK;

  bf16x8 qf[NDS];                                    // Q[query][16 ds + 8 hf ..], scaled into log2 units
  {
    const u16* qn = reinterpret_cast<const u16*>(p.qn) + (size_t)qrow * p.ldqn + (size_t)h * (p.dim_p + p.rot_p);
    const u16* qr = reinterpret_cast<const u16*>(p.qr) + (size_t)qrow * p.ldqr + (size_t)h * p.qr_head + p.qr_at;
#pragma unroll
    for (int ds = 0; ds < NDS; ++ds) {
      const int c = min(ds, nds - 1) * 16 + 8 * hf;
      float f[8];
      unpack8(ld128(c < p.dim_p ? qn + c : qr + c - p.dim_p), f);
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] = ds < nds ? f[j] * sl2 : 0.f;
      qf[ds] = as_bf16x8(pack8(f));
    }
  }
  f32x16 oacc[NDT];
#pragma unroll
  for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
    for (int i = 0; i < 16; ++i) oacc[dt][i] = 0.f;
  float m_run = 0.f, l_run = 0.f;

  const int kc = dk / 8, vc = vdk / 8, nc = p.dim_p / 8;
  const u16* kv = reinterpret_cast<const u16*>(p.kv) + (size_t)t0 * p.ldkv;
  const u16* kn = kv + (size_t)h * p.dim_p;
  const u16* vn = kv + (size_t)p.H * p.dim_p + (size_t)h * vdk;
  const u16* kr = p.krot + (size_t)t0 * p.rot_p;
  // thread's pieces: K row i / kc chunk i % kc, V likewise (the context is padded to whole tiles)
  int ko[LK], kl[LK], vo[LV], vl[LV];
  bool krt[LK];
#pragma unroll
  for (int i = 0; i < LK; ++i) {
    const int x = min(stid + i * 256, kPK * kc - 1), r = x / kc, c = x % kc;
    krt[i] = c >= nc;
    ko[i] = krt[i] ? r * p.rot_p + (c - nc) * 8 : r * p.ldkv + c * 8;
    kl[i] = r * ks + c * 16;
  }
#pragma unroll
  for (int i = 0; i < LV; ++i) {
    const int x = min(stid + i * 256, kPK * vc - 1), r = x / vc, c = x % vc;
    vo[i] = r * p.ldkv + c * 8;
    vl[i] = kPK * ks + r * vs + c * 16;
  }
  uint4 rk[LK], rv[LV];
  auto load_tile = [&](int t) {
    const u16* a = kn + (size_t)t * kPK * p.ldkv;
    const u16* b = kr + (size_t)t * kPK * p.rot_p;
    const u16* c = vn + (size_t)t * kPK * p.ldkv;
#pragma unroll
    for (int i = 0; i < LK; ++i) rk[i] = ld128((krt[i] ? b : a) + ko[i]);
#pragma unroll
    for (int i = 0; i < LV; ++i) rv[i] = ld128(c + vo[i]);
  };
  auto store_tile = [&](int stg) {                   // (pieces past the tile repeat its last one)
    unsigned char* d = simg + stg * tile_b;
#pragma unroll
    for (int i = 0; i < LK; ++i) *reinterpret_cast<uint4*>(d + kl[i]) = rk[i];
#pragma unroll
    for (int i = 0; i < LV; ++i) *reinterpret_cast<uint4*>(d + vl[i]) = rv[i];
  };
  // MFMA row R of a tile = key a_key(R): lane half hf then holds keys (i & 7) + 16 (i >> 3) + 8 hf in register i
  const int a_hi = (col >> 2) & 1, a_r = (col & 3) + 4 * (col >> 3);
  const int a_off = ((a_r & 7) + 16 * (a_r >> 3) + 8 * a_hi) * ks + hf * 16;
  const int grp = lane >> 4;
  const int v_off = kPK * ks + (8 * (grp >> 1) + ((lane >> 2) & 3)) * vs + (16 * (grp & 1) + 4 * (lane & 3)) * 2;
  const int iters = (nt + kNS - 1) / kNS;
  if (split < nt) {
    load_tile(split);
    store_tile(0);
    if (split + kNS < nt) load_tile(split + kNS);
  }
  __syncthreads();
  bool first = true;
  for (int it = 0; it < iters; ++it) {
    const int t = it * kNS + split;
    if (t < nt) {
      const int k0 = t * kPK;
      const unsigned char* img = simg + (it & 1) * tile_b;
      f32x16 s;
#pragma unroll
      for (int i = 0; i < 16; ++i) s[i] = 0.f;
#pragma unroll
      for (int ds = 0; ds < NDS; ++ds)
        s = mfma32(as_bf16x8(*reinterpret_cast<const uint4*>(img + a_off + min(ds, nds - 1) * 32)), qf[ds], s);
      if (k0 + kPK - 1 > qw0) {                      // (reaches past the wave's first query, or past the context)
#pragma unroll
        for (int i = 0; i < 16; ++i)
          if (k0 + (i & 7) + 16 * (i >> 3) + 8 * hf > qpos) s[i] = -INFINITY;
      }
      float tm = vmax3(s[0], s[1], s[2]), tn = vmax3(s[3], s[4], s[5]);
#pragma unroll
      for (int i = 6; i < 14; i += 4) {
        tm = vmax3(tm, s[i], s[i + 1]);
        tn = vmax3(tn, s[i + 2], s[i + 3]);
      }
      const float tmax = max_halves(vmax3(tm, tn, vmax3(s[14], s[15], s[15])));
      const bool move = (first && tmax != -INFINITY) || (tmax - m_run > kRescale);
      if (__any(move)) {
        const float m_new = move ? tmax : m_run;
        const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
        m_run = m_new;
        l_run *= alpha;
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) oacc[dt] *= alpha;
      }
      first = first && tmax == -INFINITY;
      float ls[4] = {0.f, 0.f, 0.f, 0.f};
      bf16x8 pb[2];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        float pf[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          pf[j] = __builtin_amdgcn_exp2f(s[8 * k + j] - m_run);
          ls[j & 3] += pf[j];
        }
        pb[k] = as_bf16x8(pack8(pf));
      }
      l_run += (ls[0] + ls[1]) + (ls[2] + ls[3]);
#pragma unroll
      for (int k = 0; k < 2; ++k)
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt) {
          if (dt * 32 >= vdk) continue;
          const unsigned char* a = img + v_off + 16 * k * vs + dt * 64;
          const uint2 lo = lds_tr16(a), hi = lds_tr16(a + 4 * vs);
          oacc[dt] = mfma32(as_bf16x8(make_uint4(lo.x, lo.y, hi.x, hi.y)), pb[k], oacc[dt]);
        }
      if (t + kNS < nt) {
        store_tile((it + 1) & 1);
        if (t + 2 * kNS < nt) load_tile(t + 2 * kNS);
      }
    }
    __syncthreads();
  }
  // ---- merge the splits (the images are free after the last barrier)
  constexpr int MO = 64 * (NDT * 16 + 2);
  float* mo = reinterpret_cast<float*>(smem) + w * MO;
  if (split > 0) {
#pragma unroll
    for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
      for (int i = 0; i < 16; ++i)
        if (dt * 32 < vdk) mo[(dt * 16 + i) * 64 + lane] = oacc[dt][i];
    const int nd = (vdk + 31) / 32;
    mo[(nd * 16) * 64 + lane] = first ? -INFINITY : m_run;
    mo[(nd * 16 + 1) * 64 + lane] = l_run;
  }
  __syncthreads();
  if (split > 0) return;
  const int nd = (vdk + 31) / 32;
  const float sink = p.sink[h] * kLog2e;
  const float m0 = first ? -INFINITY : m_run, m1 = mo[(nd * 16) * 64 + lane], M = fmaxf(sink, fmaxf(m0, m1));
  const float a0 = __builtin_amdgcn_exp2f(m0 - M), a1 = __builtin_amdgcn_exp2f(m1 - M);
  const float l = sum_halves(l_run * a0 + mo[(nd * 16 + 1) * 64 + lane] * a1);
  const float inv = 1.f / (l + __builtin_amdgcn_exp2f(sink - M));
  if (qi >= nq) return;
  // lane (col, hf) holds O^T[32 dt + (i & 3) + 8 (i >> 2) + 4 hf][query]
  const u16* gate = reinterpret_cast<const u16*>(p.gate) + (size_t)qrow * p.ldg + (size_t)h * p.vd;
  u16* out = reinterpret_cast<u16*>(p.out) + (size_t)qrow * p.ldo + (size_t)h * p.vd;
#pragma unroll
  for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
    for (int g = 0; g < 4; ++g) {
      const int d = 32 * dt + 8 * g + 4 * hf;
      if (d >= p.vd) continue;
      float gt[4], o[4];
      ld4(gate + d, gt);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int i = 4 * g + j;
        o[j] = (oacc[dt][i] * a0 + mo[(dt * 16 + i) * 64 + lane] * a1) * inv * sigm(gt[j]);
      }
      st4(out + d, o);
    }
}

constexpr size_t kMaxLds = 160 * 1024 - 2048;

template <int NDS, int NDT>
int launch(const LatentPrefillParams& p, hipStream_t st, bool only_fit) {
  const size_t lds = prefill_lds(p.dim_p + p.rot_p, p.vdk, NDT);
  if (lds > kMaxLds) return -10;
  if (only_fit) return 0;
  hipLaunchKernelGGL((latent_prefill_kernel<NDS, NDT>), dim3(p.n_tiles * p.H), dim3(256 * kNS), lds, st, p);
  return (int)hipGetLastError();
}

template <int NDS>
int dispatch_v(const LatentPrefillParams& p, hipStream_t st, bool only_fit) {
  if (p.vdk <= 64) return launch<NDS, 2>(p, st, only_fit);
  if (p.vdk <= 128) return launch<NDS, 4>(p, st, only_fit);
  if (NDS <= 12 && p.vdk <= 192) return launch<(NDS <= 12 ? NDS : 12), 6>(p, st, only_fit);
  return -10;
}

int dispatch(const LatentPrefillParams& p, hipStream_t st, bool only_fit) {
  const int nds = (p.dim_p + p.rot_p) / 16;
  if (p.dim_p < 32 || p.rot_p < 32 || p.dim_p % 32 || p.rot_p % 32 || p.vdk % 32 || p.vdk < 32) return -10;
  if (nds <= 4) return dispatch_v<4>(p, st, only_fit);
  if (nds <= 8) return dispatch_v<8>(p, st, only_fit);
  if (nds <= 12) return dispatch_v<12>(p, st, only_fit);
  if (nds <= 16) return dispatch_v<16>(p, st, only_fit);
  return -10;
}

}  // namespace

extern "C" int vwa_latent_prefill_fits(int dim_p, int rot_p, int vdk) {
  LatentPrefillParams p{};
  p.dim_p = dim_p;
  p.rot_p = rot_p;
  p.vdk = vdk;
  return dispatch(p, nullptr, true) == 0;
}

extern "C" int vwa_latent_gather(const LatentPrefillParams* p, hipStream_t st) {
  if (p->n_segs < 1 || !p->segs || p->rank_p % 32 || p->rot_p % 32 || p->kp % 8 || p->kp < p->rank_p || p->block_size < 16 ||
      (p->block_size & (p->block_size - 1)))
    return -1;
  hipLaunchKernelGGL(latent_gather_kernel, dim3(p->n_segs * 4), dim3(256), 0, st, *p);
  return (int)hipGetLastError();
}

extern "C" int vwa_latent_prefill(const LatentPrefillParams* p, hipStream_t st) {
  if (p->n_tiles < 1 || p->H < 1 || !p->q_tiles || p->ldqn % 8 || p->ldqr % 8 || p->qr_head % 8 || p->qr_at % 8 || p->ldkv % 8 ||
      p->ldg % 4 || p->ldo % 4 || p->vd % 4 || p->vd > p->vdk || (int64_t)kPK * p->ldkv >= (1ll << 31))
    return -1;
  return dispatch(*p, st, false);
}
