// Row kernels of layer stacks with an f32 residual stream.
//
//  layernorm_f32 : y (T) = (x - mean) * rstd * w (+ b) of f32 rows, two-pass statistics in f32
//  add_norm      : x += norm(branch) * w1, h = norm(x) * w2 -- the end of a sublayer and the start of the next
//  embedding_f32 : f32 residual rows from a T table, scaled
//  qkv_cache     : partial rotation of q / k heads + paged cache write (V transposed inside a block)
//  qkv_mingru    : qkv_cache and the recurrence's rows form of a decode step in one launch
#include "mixer_kernels.h"
#include "recurrence.h"

using namespace vwa;

namespace {

VWA_DEVICE float block_sum(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();  // (red may still be read from the previous sum)
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}

// one workgroup per row, the row held in registers: STEPS x 1024 columns, 4 per thread and step, all
// loads in flight at once (columns past the row repeat its last quad and count as zero)
constexpr int kLnSteps = 8;
template <class T, int STEPS>
__global__ __launch_bounds__(256) void layernorm_f32_kernel(const float* __restrict__ x, int ldx,
                                                            const float* __restrict__ w, const float* __restrict__ b,
                                                            T* __restrict__ y, int ldy, int D, int Dpad, float eps) {
  __shared__ float red[4];
  const float* xr = x + (size_t)blockIdx.x * ldx;
  T* yr = y + (size_t)blockIdx.x * ldy;
  float v[STEPS][4];
  const int last = (D - 1) & ~3;
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const float4 f = *reinterpret_cast<const float4*>(xr + min((i * 256 + (int)threadIdx.x) * 4, last));
    v[i][0] = f.x;
    v[i][1] = f.y;
    v[i][2] = f.z;
    v[i][3] = f.w;
  }
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      v[i][j] = c + j < D ? v[i][j] : 0.f;
      s += v[i][j];
    }
  }
  const float mu = block_sum(s, red) / (float)D;
  float q = 0.f;
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float d = c + j < D ? v[i][j] - mu : 0.f;
      q += d * d;
    }
  }
  const float rstd = 1.f / sqrtf(block_sum(q, red) / (float)D + eps);
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
    if (c >= D) continue;
    float o[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int cj = min(c + j, D - 1);
      o[j] = c + j < D ? (v[i][j] - mu) * rstd * w[cj] + (b ? b[cj] : 0.f) : 0.f;
    }
    st4(yr + c, o);
  }
  for (int c = ((D + 3) & ~3) + threadIdx.x; c < Dpad; c += 256) stv(yr + c, 0.f);
}

template <class T>
void launch_ln(const float* x, int ldx, const float* w, const float* b, T* y, int ldy, int rows, int D, int Dpad, float eps,
               hipStream_t st) {
  const dim3 grid(rows), block(256);
  if (D <= 1024) hipLaunchKernelGGL((layernorm_f32_kernel<T, 1>), grid, block, 0, st, x, ldx, w, b, y, ldy, D, Dpad, eps);
  else if (D <= 2048) hipLaunchKernelGGL((layernorm_f32_kernel<T, 2>), grid, block, 0, st, x, ldx, w, b, y, ldy, D, Dpad, eps);
  else if (D <= 4096) hipLaunchKernelGGL((layernorm_f32_kernel<T, 4>), grid, block, 0, st, x, ldx, w, b, y, ldy, D, Dpad, eps);
  else hipLaunchKernelGGL((layernorm_f32_kernel<T, 8>), grid, block, 0, st, x, ldx, w, b, y, ldy, D, Dpad, eps);
}

// mean and 1 / std of the row held as STEPS x 4 values per thread (columns past D are zero)
template <int STEPS>
VWA_DEVICE float2 row_stats(const float (&v)[STEPS][4], int D, float eps, float* red) {
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < STEPS; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) s += v[i][j];
  const float mu = block_sum(s, red) / (float)D;
  float q = 0.f;
#pragma unroll
  for (int i = 0; i < STEPS; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float d = (i * 256 + (int)threadIdx.x) * 4 + j < D ? v[i][j] - mu : 0.f;
      q += d * d;
    }
  return make_float2(mu, 1.f / sqrtf(block_sum(q, red) / (float)D + eps));
}

// four weights from column c (0 past D)
VWA_DEVICE void w4(const float* w, int c, int D, float (&v)[4]) {
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = c + j < D ? w[min(c + j, D - 1)] : 0.f;
}

// one workgroup per row: x += norm(sum of the branch rows) * w1; h = norm(x) * w2.  Loads of the branch,
// of the residual and of the weights are in flight together.
template <class T, int STEPS>
__global__ __launch_bounds__(256) void add_norm_kernel(float* __restrict__ x, int ldx, const T* __restrict__ br, int ldb,
                                                       int n_parts, const float* __restrict__ w1, const float* __restrict__ w2,
                                                       T* __restrict__ h, int ldh, int D, int Dpad, float eps) {
  __shared__ float red[4];
  float* xr = x + (size_t)blockIdx.x * ldx;
  const T* b = br + (size_t)blockIdx.x * n_parts * ldb;
  const int last = (D - 1) & ~3;
  float v[STEPS][4], xs[STEPS][4], wa[STEPS][4], wb[STEPS][4];
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = min((i * 256 + (int)threadIdx.x) * 4, last);
    ld4(b + c, v[i]);
    ld4(xr + c, xs[i]);
  }
  auto weights = [&](const float* w, float (&o)[STEPS][4]) {
    if (D % 4 == 0) {
#pragma unroll
      for (int i = 0; i < STEPS; ++i) ld4(w + min((i * 256 + (int)threadIdx.x) * 4, last), o[i]);
    } else {
#pragma unroll
      for (int i = 0; i < STEPS; ++i) w4(w, (i * 256 + (int)threadIdx.x) * 4, D, o[i]);
    }
  };
  weights(w1, wa);
  weights(w2 ? w2 : w1, wb);
  for (int k = 1; k < n_parts; k += 3) {
    float u[3][STEPS][4];
#pragma unroll
    for (int e = 0; e < 3; ++e)
#pragma unroll
      for (int i = 0; i < STEPS; ++i)
        ld4(b + (size_t)min(k + e, n_parts - 1) * ldb + min((i * 256 + (int)threadIdx.x) * 4, last), u[e][i]);
#pragma unroll
    for (int e = 0; e < 3; ++e)
#pragma unroll
      for (int i = 0; i < STEPS; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) v[i][j] += k + e < n_parts ? u[e][i][j] : 0.f;
  }
#pragma unroll
  for (int i = 0; i < STEPS; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if ((i * 256 + (int)threadIdx.x) * 4 + j >= D) v[i][j] = xs[i][j] = 0.f;
  const float2 sb = row_stats<STEPS>(v, D, eps, red);
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) xs[i][j] += c + j < D ? (v[i][j] - sb.x) * sb.y * wa[i][j] : 0.f;
    if (c < D) st4(xr + c, xs[i]);  // (columns past D of the last quad stay zero)
  }
  if (!w2) return;
  T* hr = h + (size_t)blockIdx.x * ldh;
  const float2 sx = row_stats<STEPS>(xs, D, eps, red);
#pragma unroll
  for (int i = 0; i < STEPS; ++i) {
    const int c = (i * 256 + threadIdx.x) * 4;
    if (c >= D) continue;
    float o[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = c + j < D ? (xs[i][j] - sx.x) * sx.y * wb[i][j] : 0.f;
    st4(hr + c, o);
  }
  for (int c = ((D + 3) & ~3) + threadIdx.x; c < Dpad; c += 256) stv(hr + c, 0.f);
}

template <class T>
void launch_add_norm(float* x, int ldx, const T* br, int ldb, int parts, const float* w1, const float* w2, T* h, int ldh,
                     int rows, int D, int Dpad, float eps, hipStream_t st) {
  const dim3 grid(rows), block(256);
  if (D <= 1024) hipLaunchKernelGGL((add_norm_kernel<T, 1>), grid, block, 0, st, x, ldx, br, ldb, parts, w1, w2, h, ldh, D, Dpad, eps);
  else if (D <= 2048) hipLaunchKernelGGL((add_norm_kernel<T, 2>), grid, block, 0, st, x, ldx, br, ldb, parts, w1, w2, h, ldh, D, Dpad, eps);
  else if (D <= 4096) hipLaunchKernelGGL((add_norm_kernel<T, 4>), grid, block, 0, st, x, ldx, br, ldb, parts, w1, w2, h, ldh, D, Dpad, eps);
  else hipLaunchKernelGGL((add_norm_kernel<T, 8>), grid, block, 0, st, x, ldx, br, ldb, parts, w1, w2, h, ldh, D, Dpad, eps);
}

template <class T>
__global__ __launch_bounds__(256) void embedding_f32_kernel(const int* __restrict__ ids, const T* __restrict__ table,
                                                            int ld, float* __restrict__ out, int ldo, int D, int Dpad,
                                                            int vocab, float scale) {
  const int row = blockIdx.x;
  const int id = ids[row];
  const bool ok = id >= 0 && id < vocab;
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c < Dpad)
    out[(size_t)row * ldo + c] = ok && c < D ? ldv(table + (size_t)id * ld + c) * scale : 0.f;
}

// Part of one row.  VEC consecutive dimensions per thread (8 when the half rotation is a
// multiple of 8, else 1): a rotated chunk reads its partner chunk rot_dims / 2 away.
template <class T, int VEC>
VWA_DEVICE void qkv_cache_row(const QkvCacheParams& p, int row, int part, int parts) {
  const T* x = reinterpret_cast<const T*>(p.x) + (size_t)row * p.ldx;
  const int64_t slot = p.slots[row];
  const int pos = min(max(p.positions[row], 0), p.max_pos - 1);
  const int64_t blk = slot >= 0 ? slot / p.block_size : 0;
  const int off = slot >= 0 ? (int)(slot % p.block_size) : 0;
  const int half = p.rot_dims >> 1;
  const float* cs = p.rope + (size_t)pos * p.rot_dims;
  const int cph = p.dk / VEC, nqk = (p.H + p.G) * cph;
  T* kc = reinterpret_cast<T*>(p.k) + blk * p.k_sb + (int64_t)off * p.dk;
  for (int u = part * 256 + threadIdx.x; u < nqk; u += parts * 256) {
    const int head = u / cph, e = (u % cph) * VEC;
    const T* xh = x + head * p.dk;
    float o[VEC];
    if (e < p.rot_dims) {
      const bool hi = e >= half;
      const int i0 = hi ? e - half : e, pe = hi ? e - half : e + half;
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        const float a = ldv(xh + e + j), b = ldv(xh + pe + j);
        const float c = cs[2 * (i0 + j)], s = cs[2 * (i0 + j) + 1];
        o[j] = hi ? a * c + b * s : a * c - b * s;
      }
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = ldv(xh + e + j);
    }
    T* dst;
    if (head < p.H) {
      dst = reinterpret_cast<T*>(p.q_out) + (size_t)row * p.ldq + head * p.dk + e;
    } else {
      if (slot < 0) continue;
      dst = kc + (int64_t)(head - p.H) * p.k_sh + e;
    }
    if constexpr (VEC == 8) {
      const float lo[4] = {o[0], o[1], o[2], o[3]}, hi4[4] = {o[4], o[5], o[6], o[7]};
      st4(dst, lo);
      st4(dst + 4, hi4);
    } else {
      stv(dst, o[0]);
    }
  }
  if (slot < 0) return;
  const T* xv = x + (p.H + p.G) * p.dk;
  T* vc = reinterpret_cast<T*>(p.v) + blk * p.v_sb + off;
  for (int u = part * 256 + threadIdx.x; u < p.G * p.dv; u += parts * 256) {
    const int g = u / p.dv, d = u % p.dv;
    vc[(int64_t)g * p.v_sh + (int64_t)d * p.block_size] = xv[u];
  }
}

template <class T, int VEC>
__global__ __launch_bounds__(256) void qkv_cache_kernel(QkvCacheParams p) {
  qkv_cache_row<T, VEC>(p, blockIdx.x, blockIdx.y, gridDim.y);
}

// grid.y: kQkvParts parts of the row's heads, then its recurrence channels by 256
constexpr int kQkvParts = 4;
template <class T, int VEC>
__global__ __launch_bounds__(256) void qkv_mingru_kernel(QkvCacheParams p, MinGruParams g) {
  if (blockIdx.y < kQkvParts) qkv_cache_row<T, VEC>(p, blockIdx.x, blockIdx.y, kQkvParts);
  else mingru_row<T>(g, blockIdx.x, (blockIdx.y - kQkvParts) * 256 + threadIdx.x);
}

}  // namespace

extern "C" int vwa_layernorm_f32(const float* x, int ldx, const float* w, const float* b, void* y, int ldy, int rows,
                                 int D, int Dpad, float eps, int f32, hipStream_t st) {
  if (rows < 1 || D < 1 || D > kLnSteps * 1024 || Dpad < D || ldx % 4 || ldy % 4 || ldx < ((D + 3) & ~3) || ldy < Dpad ||
      Dpad % 4)
    return -1;
  if (f32) launch_ln(x, ldx, w, b, reinterpret_cast<float*>(y), ldy, rows, D, Dpad, eps, st);
  else launch_ln(x, ldx, w, b, reinterpret_cast<u16*>(y), ldy, rows, D, Dpad, eps, st);
  return (int)hipGetLastError();
}

extern "C" int vwa_add_norm(float* x, int ldx, const void* br, int ldb, int n_parts, const float* w1, const float* w2, void* h,
                            int ldh, int rows, int D, int Dpad, float eps, int f32, hipStream_t st) {
  const int q = (D + 3) & ~3;
  if (rows < 1 || D < 1 || D > kLnSteps * 1024 || n_parts < 1 || ldx % 4 || ldb % 4 || ldx < q || ldb < q || !w1) return -1;
  if (w2 && (Dpad < q || Dpad % 4 || ldh % 4 || ldh < Dpad)) return -2;
  if (f32)
    launch_add_norm(x, ldx, reinterpret_cast<const float*>(br), ldb, n_parts, w1, w2, reinterpret_cast<float*>(h), ldh, rows, D,
                    Dpad, eps, st);
  else
    launch_add_norm(x, ldx, reinterpret_cast<const u16*>(br), ldb, n_parts, w1, w2, reinterpret_cast<u16*>(h), ldh, rows, D,
                    Dpad, eps, st);
  return (int)hipGetLastError();
}

extern "C" int vwa_embedding_f32(const int* ids, const void* table, int ld, float* out, int ldo, int rows, int D, int Dpad,
                                 int vocab, float scale, int f32, hipStream_t st) {
  if (rows < 1 || D < 1 || ld < D || Dpad < D || ldo < Dpad) return -1;
  if (f32)
    hipLaunchKernelGGL((embedding_f32_kernel<float>), dim3(rows, (Dpad + 255) / 256), dim3(256), 0, st, ids,
                       reinterpret_cast<const float*>(table), ld, out, ldo, D, Dpad, vocab, scale);
  else
    hipLaunchKernelGGL((embedding_f32_kernel<u16>), dim3(rows, (Dpad + 255) / 256), dim3(256), 0, st, ids,
                       reinterpret_cast<const u16*>(table), ld, out, ldo, D, Dpad, vocab, scale);
  return (int)hipGetLastError();
}

namespace {
int check_qkv(const QkvCacheParams* p) {
  return p->rows < 1 || p->H < 1 || p->G < 1 || p->dk < 1 || p->dv < 1 || p->rot_dims % 2 || p->rot_dims > p->dk ||
         p->max_pos < 1 || p->block_size < 1;
}
bool qkv_vec(const QkvCacheParams* p) {
  return (p->rot_dims / 2) % 8 == 0 && p->dk % 8 == 0 && p->ldq % 8 == 0 && p->ldx % 8 == 0;
}
}  // namespace

extern "C" int vwa_qkv_cache(const QkvCacheParams* p, hipStream_t st) {
  if (check_qkv(p)) return -1;
  const bool vec = qkv_vec(p);
  const dim3 grid(p->rows, p->rows <= 64 ? kQkvParts : 1), block(256);
  if (p->f32) {
    if (vec) hipLaunchKernelGGL((qkv_cache_kernel<float, 8>), grid, block, 0, st, *p);
    else hipLaunchKernelGGL((qkv_cache_kernel<float, 1>), grid, block, 0, st, *p);
  } else {
    if (vec) hipLaunchKernelGGL((qkv_cache_kernel<u16, 8>), grid, block, 0, st, *p);
    else hipLaunchKernelGGL((qkv_cache_kernel<u16, 1>), grid, block, 0, st, *p);
  }
  return (int)hipGetLastError();
}

extern "C" int vwa_qkv_mingru(const QkvCacheParams* p, const MinGruParams* g, hipStream_t st) {
  if (check_qkv(p) || g->rows != p->rows || g->width < 1 || g->f32 != p->f32) return -1;
  const bool vec = qkv_vec(p);
  const dim3 grid(p->rows, kQkvParts + (g->width + 255) / 256), block(256);
  if (p->f32) {
    if (vec) hipLaunchKernelGGL((qkv_mingru_kernel<float, 8>), grid, block, 0, st, *p, *g);
    else hipLaunchKernelGGL((qkv_mingru_kernel<float, 1>), grid, block, 0, st, *p, *g);
  } else {
    if (vec) hipLaunchKernelGGL((qkv_mingru_kernel<u16, 8>), grid, block, 0, st, *p, *g);
    else hipLaunchKernelGGL((qkv_mingru_kernel<u16, 1>), grid, block, 0, st, *p, *g);
  }
  return (int)hipGetLastError();
}
