// Gated recurrences (f32 state per sequence and channel, one state slot per live sequence).
//
// minGRU: z = sigmoid(zp + zb), u = xp + xb, S <- (1 - z) S + z * (u >= 0 ? u + 1/2 : sigmoid(u)),
// out = S * silu(gp) * out_scale.  The gates read only the current token, so a run of tokens is a
// first-order linear scan per channel:
//
//  * rows form (decode steps, <= 64 rows): one workgroup per (256 channels, run of rows of one
//    sequence); the run's head row walks it token by token;
//  * scan form (prompt-sized runs): runs are cut into chunks.  Launch 1 reduces each chunk to
//    S_end = A S_start + B (and takes a copy of the run's initial state); launch 2 folds the chunks
//    in front of its own, then walks its tokens and writes the outputs; the run's last chunk
//    writes the state back.  Two streaming passes over the projections, all chunks in parallel.
//
// A run that starts at position 0 starts from a zero state whatever the slot holds.
#include "recurrence.h"

using namespace vwa;

namespace {

template <class T>
__global__ __launch_bounds__(256) void mingru_rows_kernel(MinGruParams p) {
  mingru_row<T>(p, blockIdx.y, blockIdx.x * 256 + threadIdx.x);
}

// VEC consecutive channels of one row
template <class T, int VEC> VWA_DEVICE void ldc(const T* p, float (&v)[VEC]) {
  if constexpr (VEC == 1) {
    v[0] = ldv(p);
  } else if constexpr (sizeof(T) == 2) {
    const unsigned u = *reinterpret_cast<const unsigned*>(p);
    v[0] = __uint_as_float(u << 16);
    v[1] = __uint_as_float(u & 0xffff0000u);
  } else {
    const float2 u = *reinterpret_cast<const float2*>(p);
    v[0] = u.x;
    v[1] = u.y;
  }
}

constexpr int kScanBatch = 8;  // rows whose loads are in flight together, a batch ahead of the arithmetic

// PASS 1: per (chunk, channel) A = prod (1 - z), B = the chunk's end state from a zero start
// PASS 2: outputs (and the state of a run's last chunk)
template <class T, int PASS, int VEC>
__global__ __launch_bounds__(256) void mingru_scan_kernel(MinGruParams p) {
  const int ck = blockIdx.y;
  const int ch = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (ch >= p.width) return;
  const bool two = VEC == 2 && ch + 1 < p.width;  // (an odd width: the second channel is padding)
  const int row0 = p.chunks[4 * ck], n = p.chunks[4 * ck + 1], idx = p.chunks[4 * ck + 2], cnt = p.chunks[4 * ck + 3];
  const T* z = reinterpret_cast<const T*>(p.z) + ch + (size_t)row0 * p.ld;
  const T* x = reinterpret_cast<const T*>(p.x) + ch + (size_t)row0 * p.ld;
  const T* g = reinterpret_cast<const T*>(p.g) + ch + (size_t)row0 * p.ld;
  float zb[VEC], xb[VEC], S[VEC], A[VEC];
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    const int c = min(ch + e, p.width - 1);
    zb[e] = p.zb ? p.zb[c] : 0.f;
    xb[e] = p.xb ? p.xb[c] : 0.f;
    S[e] = 0.f;
    A[e] = 1.f;
  }
  float bz[2][kScanBatch][VEC], bx[2][kScanBatch][VEC], bg[2][kScanBatch][VEC];
  auto load = [&](int q, int t0) {
#pragma unroll
    for (int t = 0; t < kScanBatch; ++t) {
      const size_t o = (size_t)min(t0 + t, n - 1) * p.ld;
      ldc<T, VEC>(z + o, bz[q][t]);
      ldc<T, VEC>(x + o, bx[q][t]);
      if (PASS == 2) ldc<T, VEC>(g + o, bg[q][t]);
    }
  };
  load(0, 0);
  float* st = p.state + (size_t)p.seq_ids[row0] * p.state_ld + ch;
  const size_t W = p.width;
  if constexpr (PASS == 2) {
    const int first = ck - idx;
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      if (e && !two) break;
      S[e] = p.cS[first * W + ch + e];
#pragma unroll 16
      for (int k = first; k < ck; ++k) S[e] = p.cA[k * W + ch + e] * S[e] + p.cB[k * W + ch + e];
    }
  }
  T* out = reinterpret_cast<T*>(p.out) + (size_t)row0 * p.ldo + ch;
  auto work = [&](int q, int t0) {
#pragma unroll
    for (int t = 0; t < kScanBatch; ++t) {
      if (t0 + t >= n) break;
      float o[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        const Gate gt = min_gru_gate(bz[q][t][e] + zb[e], bx[q][t][e] + xb[e]);
        A[e] *= 1.f - gt.z;
        S[e] = (1.f - gt.z) * S[e] + gt.z * gt.c;
        o[e] = PASS == 2 ? S[e] * silu(bg[q][t][e]) * p.out_scale : 0.f;
      }
      if constexpr (PASS == 2) {
        T* y = out + (size_t)(t0 + t) * p.ldo;
        stv(y, o[0]);
        if constexpr (VEC == 2) {
          if (two) stv(y + 1, o[VEC - 1]);
        }
      }
    }
  };
  for (int t0 = 0; t0 < n; t0 += 2 * kScanBatch) {
    if (t0 + kScanBatch < n) load(1, t0 + kScanBatch);
    work(0, t0);
    if (t0 + kScanBatch >= n) break;
    if (t0 + 2 * kScanBatch < n) load(0, t0 + 2 * kScanBatch);
    work(1, t0 + kScanBatch);
  }
#pragma unroll
  for (int e = 0; e < VEC; ++e) {
    if (e && !two) break;
    if constexpr (PASS == 1) {
      p.cA[ck * W + ch + e] = A[e];
      p.cB[ck * W + ch + e] = S[e];
      if (idx == 0) p.cS[ck * W + ch + e] = p.positions[row0] > 0 ? st[e] : 0.f;
    } else {
      if (idx == cnt - 1) st[e] = S[e];
    }
  }
}

template <class T, int VEC>
void launch_scan(const MinGruParams& p, hipStream_t st) {
  const dim3 grid((p.width + 256 * VEC - 1) / (256 * VEC), p.n_chunks), block(256);
  hipLaunchKernelGGL((mingru_scan_kernel<T, 1, VEC>), grid, block, 0, st, p);
  hipLaunchKernelGGL((mingru_scan_kernel<T, 2, VEC>), grid, block, 0, st, p);
}

}  // namespace

extern "C" int vwa_mingru_rows(const MinGruParams* p, hipStream_t st) {
  if (p->rows < 1 || p->width < 1) return -1;
  const dim3 grid((p->width + 255) / 256, p->rows), block(256);
  if (p->f32) hipLaunchKernelGGL((mingru_rows_kernel<float>), grid, block, 0, st, *p);
  else hipLaunchKernelGGL((mingru_rows_kernel<u16>), grid, block, 0, st, *p);
  return (int)hipGetLastError();
}

extern "C" int vwa_mingru_scan(const MinGruParams* p, hipStream_t st) {
  if (p->rows < 1 || p->width < 1 || p->n_chunks < 1 || !p->chunks || !p->cA || !p->cB || !p->cS) return -1;
  // two channels per thread where the projections' columns pair up (4- / 8-byte loads; rows padded to it)
  const uintptr_t al = p->f32 ? 7 : 3;
  const bool pair = p->ld % 2 == 0 && !((reinterpret_cast<uintptr_t>(p->z) | reinterpret_cast<uintptr_t>(p->x) |
                                         reinterpret_cast<uintptr_t>(p->g)) & al) && p->width % 2 == 0;
  if (p->f32) pair ? launch_scan<float, 2>(*p, st) : launch_scan<float, 1>(*p, st);
  else pair ? launch_scan<u16, 2>(*p, st) : launch_scan<u16, 1>(*p, st);
  return (int)hipGetLastError();
}
