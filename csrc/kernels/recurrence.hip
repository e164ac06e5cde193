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
#include "common.h"
#include "stack_kernels.h"

using namespace vwa;

namespace {

template <class T> VWA_DEVICE float ldv(const T* p);
template <> VWA_DEVICE float ldv<u16>(const u16* p) { return bf2f(*p); }
template <> VWA_DEVICE float ldv<float>(const float* p) { return *p; }
VWA_DEVICE void stv(u16* p, float v) { *p = f2bf(v); }
VWA_DEVICE void stv(float* p, float v) { *p = v; }

VWA_DEVICE float sigm(float x) { return 1.f / (1.f + __expf(-x)); }

struct Gate {
  float z, c;
};
VWA_DEVICE Gate min_gru_gate(float zp, float u) {
  return Gate{sigm(zp), u >= 0.f ? u + 0.5f : sigm(u)};
}

template <class T>
__global__ __launch_bounds__(256) void mingru_rows_kernel(MinGruParams p) {
  const int r0 = blockIdx.y;
  const int ch = blockIdx.x * 256 + threadIdx.x;
  if (ch >= p.width) return;
  T* out = reinterpret_cast<T*>(p.out);
  if (p.slots[r0] < 0) {  // inert row of a padded step
    stv(out + (size_t)r0 * p.ldo + ch, 0.f);
    return;
  }
  const int seq = p.seq_ids[r0];
  if (r0 > 0 && p.seq_ids[r0 - 1] == seq && p.slots[r0 - 1] >= 0) return;  // not the head of its run
  const T* z = reinterpret_cast<const T*>(p.z) + ch;
  const T* x = reinterpret_cast<const T*>(p.x) + ch;
  const T* g = reinterpret_cast<const T*>(p.g) + ch;
  const float zb = p.zb ? p.zb[ch] : 0.f, xb = p.xb ? p.xb[ch] : 0.f;
  float* st = p.state + (size_t)seq * p.state_ld + ch;
  float S = p.positions[r0] > 0 ? *st : 0.f;
  for (int r = r0; r < p.rows; ++r) {
    if (r > r0 && (p.seq_ids[r] != seq || p.slots[r] < 0)) break;
    const size_t o = (size_t)r * p.ld;
    const Gate gt = min_gru_gate(ldv(z + o) + zb, ldv(x + o) + xb);
    S = (1.f - gt.z) * S + gt.z * gt.c;
    stv(out + (size_t)r * p.ldo + ch, S * silu(ldv(g + o)) * p.out_scale);
  }
  *st = S;
}

// PASS 1: per (chunk, channel) A = prod (1 - z), B = the chunk's end state from a zero start
// PASS 2: outputs (and the state of a run's last chunk)
template <class T, int PASS>
__global__ __launch_bounds__(256) void mingru_scan_kernel(MinGruParams p) {
  const int ck = blockIdx.y;
  const int ch = blockIdx.x * 256 + threadIdx.x;
  if (ch >= p.width) return;
  const int row0 = p.chunks[4 * ck], n = p.chunks[4 * ck + 1], idx = p.chunks[4 * ck + 2], cnt = p.chunks[4 * ck + 3];
  const T* z = reinterpret_cast<const T*>(p.z) + ch + (size_t)row0 * p.ld;
  const T* x = reinterpret_cast<const T*>(p.x) + ch + (size_t)row0 * p.ld;
  const T* g = reinterpret_cast<const T*>(p.g) + ch + (size_t)row0 * p.ld;
  const float zb = p.zb ? p.zb[ch] : 0.f, xb = p.xb ? p.xb[ch] : 0.f;
  float* st = p.state + (size_t)p.seq_ids[row0] * p.state_ld + ch;
  if constexpr (PASS == 1) {
    float A = 1.f, B = 0.f;
#pragma unroll 8
    for (int t = 0; t < n; ++t) {
      const Gate gt = min_gru_gate(ldv(z + (size_t)t * p.ld) + zb, ldv(x + (size_t)t * p.ld) + xb);
      A *= 1.f - gt.z;
      B = (1.f - gt.z) * B + gt.z * gt.c;
    }
    p.cA[(size_t)ck * p.width + ch] = A;
    p.cB[(size_t)ck * p.width + ch] = B;
    if (idx == 0) p.cS[(size_t)ck * p.width + ch] = p.positions[row0] > 0 ? *st : 0.f;
  } else {
    const int first = ck - idx;
    float S = p.cS[(size_t)first * p.width + ch];
#pragma unroll 4
    for (int k = first; k < ck; ++k) S = p.cA[(size_t)k * p.width + ch] * S + p.cB[(size_t)k * p.width + ch];
    T* out = reinterpret_cast<T*>(p.out) + (size_t)row0 * p.ldo + ch;
#pragma unroll 8
    for (int t = 0; t < n; ++t) {
      const Gate gt = min_gru_gate(ldv(z + (size_t)t * p.ld) + zb, ldv(x + (size_t)t * p.ld) + xb);
      S = (1.f - gt.z) * S + gt.z * gt.c;
      stv(out + (size_t)t * p.ldo, S * silu(ldv(g + (size_t)t * p.ld)) * p.out_scale);
    }
    if (idx == cnt - 1) *st = S;
  }
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
  const dim3 grid((p->width + 255) / 256, p->n_chunks), block(256);
  if (p->f32) {
    hipLaunchKernelGGL((mingru_scan_kernel<float, 1>), grid, block, 0, st, *p);
    hipLaunchKernelGGL((mingru_scan_kernel<float, 2>), grid, block, 0, st, *p);
  } else {
    hipLaunchKernelGGL((mingru_scan_kernel<u16, 1>), grid, block, 0, st, *p);
    hipLaunchKernelGGL((mingru_scan_kernel<u16, 2>), grid, block, 0, st, *p);
  }
  return (int)hipGetLastError();
}
