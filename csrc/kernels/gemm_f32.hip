// 32-bit GEMM on the f32 MFMA (v_mfma_f32_16x16x4_f32: f32 products, f32 accumulation) for models
// that run in 32-bit: Y = epi(X . W^T), both operands row-major with K contiguous.
//
// A 4-wave workgroup computes 64 x 64; each wave 32 x 32 = 2 x 2 MFMA tiles.  A lane's 16-byte load
// holds 4 consecutive k of its row; the four MFMAs of a 16-deep step take element j of every lane
// group, so A and B use the same k order and no LDS is needed.
#include "common.h"
#include "stack_kernels.h"

using namespace vwa;

namespace {

VWA_DEVICE f32x4 mfma4(float a, float b, const f32x4& c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

template <int EPI>
__global__ __launch_bounds__(256) void gemm_f32_kernel(GemmF32Params p) {
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int rl = lane & 15, g = lane >> 4;
  const int m0 = blockIdx.y * 64 + (w & 1) * 32, n0 = blockIdx.x * 64 + (w >> 1) * 32;
  if (m0 >= p.M || n0 >= p.N) return;
  // rows past the end read the last row (their results are not stored)
  const float* xa[2];
  const float* wb[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    xa[i] = p.X + (size_t)min(m0 + 16 * i + rl, p.M - 1) * p.ldx + 4 * g;
    wb[i] = p.W + (size_t)min(n0 + 16 * i + rl, p.N - 1) * p.K + 4 * g;
  }
  f32x4 acc[2][2] = {};
#pragma unroll 2
  for (int k = 0; k < p.K; k += 16) {
    float4 a[2], b[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      a[i] = *reinterpret_cast<const float4*>(xa[i] + k);
      b[i] = *reinterpret_cast<const float4*>(wb[i] + k);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        acc[i][j] = mfma4(a[i].x, b[j].x, acc[i][j]);
        acc[i][j] = mfma4(a[i].y, b[j].y, acc[i][j]);
        acc[i][j] = mfma4(a[i].z, b[j].z, acc[i][j]);
        acc[i][j] = mfma4(a[i].w, b[j].w, acc[i][j]);
      }
  }
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int m = m0 + 16 * i + 4 * g + r;
      if (m >= p.M) continue;
      if constexpr (EPI == 2) {  // (the wave's two column tiles are gate and up of the same 16 features)
        p.Y[(size_t)m * p.ldy + (n0 >> 1) + rl] = silu(acc[i][0][r]) * acc[i][1][r];
        continue;
      }
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int n = n0 + 16 * j + rl;
        if (n >= p.N) continue;
        float v = acc[i][j][r];
        if constexpr (EPI == 1) v += p.R[(size_t)m * p.ldr + n];
        if (EPI == 6 && n >= p.n_split) {
          v = fmaxf(v, 0.f);
          p.Y2[(size_t)m * p.ldy2 + n - p.n_split] = v * v;
        } else {
          p.Y[(size_t)m * p.ldy + n] = v;
        }
      }
    }
}

}  // namespace

extern "C" int vwa_gemm_f32(int epi, const GemmF32Params* p, hipStream_t st) {
  if (p->M < 1 || p->N < 1 || p->K < 16 || p->K % 16 || p->ldx % 4) return -1;
  if ((reinterpret_cast<uintptr_t>(p->X) & 15) || (reinterpret_cast<uintptr_t>(p->W) & 15)) return -2;
  if (epi == 1 && !p->R) return -3;
  if (epi == 6 && (!p->Y2 || p->n_split < 0 || p->n_split > p->N)) return -4;
  if (epi == 2 && p->N % 32) return -5;
  const dim3 grid((p->N + 63) / 64, (p->M + 63) / 64), block(256);
  switch (epi) {
    case 0: hipLaunchKernelGGL((gemm_f32_kernel<0>), grid, block, 0, st, *p); break;
    case 1: hipLaunchKernelGGL((gemm_f32_kernel<1>), grid, block, 0, st, *p); break;
    case 2: hipLaunchKernelGGL((gemm_f32_kernel<2>), grid, block, 0, st, *p); break;
    case 6: hipLaunchKernelGGL((gemm_f32_kernel<6>), grid, block, 0, st, *p); break;
    default: return -6;
  }
  return (int)hipGetLastError();
}
