// Real-gated linear recurrence behind a short causal convolution (RgLruParams), f32 state.
//
// One workgroup handles whole blocks of channels: it forms u = conv(x) of up to RT rows in LDS, multiplies
// it by the block's two gate matrices on the MFMA (D[row][channel]: a lane holds 4 consecutive rows of one
// channel) and scans S <- a S + b over the rows in registers -- in the lane, over the four lane groups,
// over the 16-row tiles.  A row that starts a run of its sequence folds the state it starts from into b and
// takes a = 0, so one scan serves any mix of runs.
//
//  * rows form (decode steps, <= 64 rows): a workgroup per block and 16 rows, for the runs that start there; runs
//    are found from the sequence ids.  It is the only reader and writer of its runs' state in the block.
//  * scan form (prompt-sized runs): workgroups per (chunk of a run, block, 128 channels).  Launch 1 forms u and
//    reduces every chunk to S_end = A S_start + B; launch 2 folds the chunks in front of its own, scans again
//    and writes the outputs; the run's last chunk writes the state.
//
// A run that starts at position 0 starts from zeros whatever its slot holds.
#include "mixer_kernels.h"
#include "stack_types.h"

using namespace vwa;

namespace {

constexpr size_t kMaxLds = 160 * 1024 - 2048;
constexpr int kPad = 16;                             // bytes between LDS rows of u: 16 rows hit different banks

// v, with nothing known about it
VWA_DEVICE int opaque(int v) {
  asm volatile("" : "+v"(v));
  return v;
}

VWA_DEVICE float rcp_sigm(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
VWA_DEVICE float gelu_tanh(float z) { return z * rcp_sigm(1.5957691216057308f * (z + 0.044715f * z * z * z)); }

struct Step {
  float a, b;
};
// The recurrence's step from the gates' pre-activations: a = exp(x), b = sqrt(1 - a^2) i u.  1 - a^2 = -expm1(2 x)
// by its series where a is near 1 (the difference would lose the small decays), directly elsewhere.
VWA_DEVICE Step lru_step(float rp, float ip, float decay, float u) {
  const float x = decay * rcp_sigm(rp), y = 2.f * x;
  const float a = __expf(x);
  float q = 1.f / 5040.f;                            // (|y| < 1/4: the next term is below 2e-9 of y)
  q = q * y + 1.f / 720.f;
  q = q * y + 1.f / 120.f;
  q = q * y + 1.f / 24.f;
  q = q * y + 1.f / 6.f;
  q = q * y + 0.5f;
  q = q * y + 1.f;
  const float d = y > -0.25f ? -y * q : 1.f - a * a;
  return Step{a, __builtin_amdgcn_sqrtf(d) * rcp_sigm(ip) * u};
}

template <class T> VWA_DEVICE int u_stride(int bs) { return bs * (int)sizeof(T) + kPad; }

// gate fragments of 16 channels, steps s0 .. s0 + PRE
template <int PRE>
struct GateFrags {
  uint4 r[PRE], i[PRE];
  template <class T> VWA_DEVICE void load(const T* gw, int steps, int s0, int beg = 0, int end = PRE) {
    const uint4* wr = reinterpret_cast<const uint4*>(gw);
    const unsigned l = lane_id();                    // (uniform bases: one offset register)
#pragma unroll
    for (int s = 0; s < PRE; ++s) {
      if (s < beg || s >= end) continue;
      const uint4* ws = wr + min(s0 + s, steps - 1) * 64;
      r[s] = ws[l];
      i[s] = (ws + steps * 64)[l];
    }
  }
};
// r, i pre-activations of 16 NT rows for 16 channels: u in LDS; f holds the first fragments
template <class T, int NT, int PRE>
VWA_DEVICE void gate_products(const char* us, int stride, const T* gw, int steps, GateFrags<PRE>& f, f32x4 (&ar)[NT], f32x4 (&ai)[NT]) {
  using M = MM<T>;
  const int lane = lane_id(), rl = lane & 15, b = lane >> 4;
#pragma unroll
  for (int t = 0; t < NT; ++t) ar[t] = ai[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  const char* ua = us + rl * stride + b * 16;
#pragma unroll 1
  for (int s0 = 0; s0 < steps; s0 += PRE) {
#pragma unroll
    for (int s = 0; s < PRE; ++s) {
      if (s0 + s < steps) {
#pragma unroll
        for (int t = 0; t < NT; ++t) {
          const uint4 a = *reinterpret_cast<const uint4*>(ua + t * 16 * stride + (s0 + s) * 64);
          ar[t] = M::mma(a, f.r[s], ar[t]);
          ai[t] = M::mma(a, f.i[s], ai[t]);
        }
      }
      if (NT == 1 && (s & 1)) __builtin_amdgcn_sched_barrier(0);  // (bounds the operands read ahead)
    }
    if (s0 + PRE < steps) f.load(gw, steps, s0 + PRE);
  }
}

// inclusive scan of the 16 rows of a tile (row 4 b + i in lane group b, register i): s[i] <- the state after
// row i given the state ``carry`` before the tile; A, B: the tile as one step.  Returns the state after it.
VWA_DEVICE float scan_tile(const float (&a)[4], const float (&bb)[4], float carry, float (&s)[4], float& A, float& B) {
  const int lane = lane_id(), g = lane >> 4;
  float pa[4], pb[4];
  pa[0] = a[0];
  pb[0] = bb[0];
#pragma unroll
  for (int i = 1; i < 4; ++i) {
    pa[i] = a[i] * pa[i - 1];
    pb[i] = a[i] * pb[i - 1] + bb[i];
  }
  // the lane groups in front: (ea, eb)
  float ea = 1.f, eb = 0.f, ta = 1.f, tb = 0.f;
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const float ka = __shfl(pa[3], (lane & 15) + 16 * k, 64), kb = __shfl(pb[3], (lane & 15) + 16 * k, 64);
    tb = ka * tb + kb;
    ta = ka * ta;
    if (k + 1 == g) {
      ea = ta;
      eb = tb;
    }
  }
  const float s0 = ea * carry + eb;
#pragma unroll
  for (int i = 0; i < 4; ++i) s[i] = pa[i] * s0 + pb[i];
  A = ta;
  B = tb;
  return ta * carry + tb;
}

// row r's inputs (without xb)
template <class T>
VWA_DEVICE const T* input_at(const RgLruParams& p, int r, int ch) {
  return reinterpret_cast<const T*>(p.yx) + (size_t)r * p.ld + p.nb * p.bs + ch;
}

// four channels of u of row r: j rows of the run lie in front of r in this step, the inputs before them come from
// the state row st (fresh: zeros).  Both places of a tap are requested, whichever it takes: no load waits for another.
template <class T, int G>
VWA_DEVICE void conv4(const RgLruParams& p, int r, int j, const float* st, bool fresh, int ch, float (&u)[4]) {
  const int W = p.nb * p.bs;
  float xb[4];
  ld4(p.cb + ch, u);
  ld4(p.xb + ch, xb);
#pragma unroll 1
  for (int k0 = 0; k0 < p.taps; k0 += G) {           // k tokens back
    float x[G][4], s[G][4], w[G][4];
#pragma unroll
    for (int e = 0; e < G; ++e) {
      const int k = min(k0 + e, p.taps - 1);
      ld4(input_at<T>(p, r - min(k, j), ch), x[e]);
      ld4(st + (size_t)min(p.taps - (k - j), p.taps - 1) * W + ch, s[e]);
      ld4(p.cw + (size_t)(p.taps - 1 - k) * W + ch, w[e]);
    }
#pragma unroll
    for (int e = 0; e < G; ++e) {
      if (k0 + e >= p.taps) break;
#pragma unroll
      for (int c = 0; c < 4; ++c) u[c] += w[e][c] * (k0 + e <= j ? x[e][c] + xb[c] : fresh ? 0.f : s[e][c]);
    }
  }
}

// the same for rows r .. r + 3, all their taps among the inputs of this step's rows r_min .. r_max
template <class T>
VWA_DEVICE void conv_strip(const RgLruParams& p, int r, int r_min, int r_max, int ch, float (&u)[4][4]) {
  const int W = p.nb * p.bs;
  float xb[4];
  ld4(p.xb + ch, xb);
#pragma unroll
  for (int i = 0; i < 4; ++i) ld4(p.cb + ch, u[i]);
#pragma unroll 1
  for (int k0 = 0; k0 < p.taps; k0 += 4) {
    float x[7][4], w[4][4];
#pragma unroll
    for (int e = 0; e < 7; ++e) ld4(input_at<T>(p, min(max(r + 3 - k0 - e, r_min), r_max), ch), x[e]);
#pragma unroll
    for (int e = 0; e < 4; ++e) ld4(p.cw + (size_t)max(p.taps - 1 - k0 - e, 0) * W + ch, w[e]);
#pragma unroll
    for (int e = 0; e < 4; ++e)
#pragma unroll
      for (int c = 0; c < 4; ++c) w[e][c] = k0 + e < p.taps ? w[e][c] : 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int c = 0; c < 4; ++c) u[i][c] += w[e][c] * (x[3 - i + e][c] + xb[c]);
  }
}

// the last taps - 1 inputs of a run of n rows ending at row r -> its state row (n rows shift the old ones)
template <class T>
VWA_DEVICE void save_inputs4(const RgLruParams& p, int r, int n, bool fresh, float* st, int ch) {
  constexpr int G = 3;
  const int W = p.nb * p.bs;
  float xb[4];
  ld4(p.xb + ch, xb);
#pragma unroll 1
  for (int i0 = 1; i0 < p.taps; i0 += G) {           // place i: the input taps - i tokens before the next one
    float x[G][4], s[G][4];
#pragma unroll
    for (int e = 0; e < G; ++e) {
      const int i = min(i0 + e, p.taps - 1), back = p.taps - 1 - i;  // rows before r
      ld4(input_at<T>(p, r - min(back, n - 1), ch), x[e]);
      ld4(st + (size_t)min(i + n, p.taps - 1) * W + ch, s[e]);       // (read before a lower place is written)
    }
#pragma unroll
    for (int e = 0; e < G; ++e) {
      const int i = i0 + e;
      if (i >= p.taps) break;
#pragma unroll
      for (int c = 0; c < 4; ++c) x[e][c] = p.taps - 1 - i < n ? x[e][c] + xb[c] : fresh ? 0.f : s[e][c];
      st4(st + (size_t)i * W + ch, x[e]);
    }
  }
}

// ------------------------------------------------------------------------------------------ rows form
// Workgroup (block, tile): the runs whose first row lies in rows 16 tile .. 16 tile + 15, 16 rows at a time to
// their ends (other runs' rows count as inert).
template <class T>
__global__ __launch_bounds__(1024) void rglru_rows_kernel(RgLruParams p) {
  constexpr int PRE = 8;
  extern __shared__ __attribute__((aligned(16))) char us[];
  // of a row: its sequence; its run's first row (-1: inert); its run's rows (at the run's last row, else 0); whether
  // tokens precede it / its run
  __shared__ int s_seq[64], s_first[64], s_len[64], s_old[64], s_run_old[64];
  const int blk = blockIdx.x, lo = blockIdx.y * 16, bs = p.bs, c0 = blk * bs;
  const int tid0 = threadIdx.x, nthr = blockDim.x, w = __builtin_amdgcn_readfirstlane(tid0 >> 6);
  const int stride = u_stride<T>(bs), steps = bs / MM<T>::KS, tiles = bs / 16, waves = nthr >> 6;
  T* out = reinterpret_cast<T*>(p.out);
  const T* gw0 = reinterpret_cast<const T*>(p.gw) + (size_t)blk * tiles * 32 * bs;
  if (tid0 < 64) {                                   // (one wave: runs from the rows' ids)
    const int r = tid0, rc = min(r, p.rows - 1), id = p.seq_ids[rc], old = p.positions[rc] > 0;
    const bool live = p.slots[rc] >= 0 && r < p.rows;
    const int seq = live ? id : -1 - r;
    const int before = __shfl_up(seq, 1, 64), after = __shfl_down(seq, 1, 64);
    const unsigned long long heads = __ballot(live && (r == 0 || before != seq));
    const unsigned long long mine = heads & ((2ull << r) - 1ull);
    const int first = live && mine ? 63 - __builtin_clzll(mine) : -1;
    s_seq[r] = max(seq, 0);
    s_first[r] = first;
    s_len[r] = live && (r == 63 || after != seq) ? r + 1 - first : 0;
    s_old[r] = old;
    s_run_old[r] = __shfl(old, max(first, 0), 64);
  }
  __syncthreads();
  const int quads = bs / 4, hi = min(lo + 16, p.rows);
  auto owned = [&](int r) { return s_first[r] >= lo && s_first[r] < hi; };
  auto state_of = [&](int r) { return p.state + (size_t)s_seq[r] * p.state_ld; };
#pragma unroll 1
  for (int r0 = lo; r0 < p.rows; r0 += 16) {
    if (r0 > lo && !owned(r0)) break;                // (a run that goes past the tile owns the next row)
    const int n = min(16, p.rows - r0);
#pragma unroll 1
    for (int t0 = 0; t0 < tiles; t0 += waves) {
      // (mostly the only pass: addresses are formed where they are used, not kept across passes)
      const int tid = opaque(tid0), lane = tid & 63, rl = lane & 15, g = lane >> 4;
      const int ct = min(t0 + w, tiles - 1), ch = c0 + ct * 16 + rl;
      // ---- requested ahead of the convolution
      const T* gw = gw0 + (size_t)ct * 32 * bs;
      GateFrags<PRE> f;
      f.load(gw, steps, 0, 0, PRE / 2);
      const float rb = p.rb[ch], ib = p.ib[ch], dec = p.decay[ch], yb = p.yb[ch];
      T yv[4];
      float s_in[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = r0 + min(4 * g + i, n - 1);
        yv[i] = reinterpret_cast<const T*>(p.yx)[(size_t)r * p.ld + ch];
        s_in[i] = state_of(r)[ch];
      }
      if (t0 == 0) {
#pragma unroll 1
        for (int x = tid; x < 16 * quads; x += nthr) {
          const int i = x / quads, c = (x % quads) * 4, r = r0 + i;
          float u[4] = {0.f, 0.f, 0.f, 0.f};
          if (i < n && owned(r)) conv4<T, 4>(p, r, r - s_first[r], state_of(r), !s_run_old[r], c0 + c, u);
          st4(reinterpret_cast<T*>(us + i * stride) + c, u);
        }
      }
      __builtin_amdgcn_sched_barrier(0);             // (the convolution's registers are free from here)
      f.load(gw, steps, 0, PRE / 2, PRE);
      __syncthreads();                               // (every read of the old inputs is done as well)
      if (t0 + w >= tiles) continue;
      f32x4 ar[1], ai[1];
      gate_products<T, 1, PRE>(us, stride, gw, steps, f, ar, ai);
      float a[4], b[4], s[4], A, B;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int li = 4 * g + i, r = r0 + min(li, n - 1);
        const bool mine = li < n && owned(r), head = s_first[r] == r || li == 0;
        const float u = ldv(reinterpret_cast<const T*>(us + li * stride) + ct * 16 + rl);
        const Step st = lru_step(ar[0][i] + rb, ai[0][i] + ib, dec, u);
        // (a run that goes on from the rows before: its state was saved)
        b[i] = !mine ? 0.f : head && s_old[r] ? st.b + st.a * s_in[i] : st.b;
        a[i] = mine && !head ? st.a : 0.f;
      }
      scan_tile(a, b, 0.f, s, A, B);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int li = 4 * g + i, r = r0 + li;
        if (li >= n) continue;
        if (owned(r)) {
          stv(out + (size_t)r * p.ldo + ch, s[i] * gelu_tanh(ldv(&yv[i]) + yb));
          if (s_len[r] > 0 || li == n - 1) state_of(r)[ch] = s[i];
        } else if (s_first[r] < 0 && r0 == lo) {
          stv(out + (size_t)r * p.ldo + ch, 0.f);    // inert row of a padded step
        }
      }
    }
#pragma unroll 1
    for (int x = opaque(tid0); x < n * quads; x += nthr) {
      const int r = r0 + x / quads, len = s_len[r];
      if (len > 0 && owned(r)) save_inputs4<T>(p, r, len, !s_run_old[r], state_of(r), c0 + (x % quads) * 4);
    }
    __syncthreads();                                 // u is overwritten; saved states are read by the next rows
  }
}

// ------------------------------------------------------------------------------------------ scan form
constexpr int kScanWaves = 8;

// Pass 1 forms u by the convolution and leaves it in p.u for pass 2.
template <class T, int PASS, int NT>
__global__ __launch_bounds__(kScanWaves * 64, NT == 4 ? 4 : 2) void rglru_scan_kernel(RgLruParams p) {
  constexpr int RT = NT * 16;
  extern __shared__ __attribute__((aligned(16))) char us[];
  const int ck = blockIdx.x, blk = blockIdx.y, bs = p.bs, W = p.nb * bs, c0 = blk * bs;
  const int tid = threadIdx.x, lane = lane_id(), w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int rl = lane & 15, g = lane >> 4, stride = u_stride<T>(bs), steps = bs / MM<T>::KS;
  const int row0 = p.chunks[4 * ck], n = p.chunks[4 * ck + 1], idx = p.chunks[4 * ck + 2], cnt = p.chunks[4 * ck + 3];
  const int run0 = idx > 0 ? p.chunks[4 * (ck - idx)] : row0;  // first row of the run
  const int ct = blockIdx.z * kScanWaves + w;
  const bool active = ct < bs / 16;
  const int ch = c0 + (active ? ct : 0) * 16 + rl;
  const T* gw = reinterpret_cast<const T*>(p.gw) + (size_t)(blk * (bs / 16) + (active ? ct : 0)) * 32 * bs;
  constexpr int PRE = 4;
  GateFrags<PRE> f;
  const int pos0 = p.positions[run0];
  float* st = p.state + (size_t)p.seq_ids[row0] * p.state_ld;
  const float rb = p.rb[ch], ib = p.ib[ch], dec = p.decay[ch], yb = p.yb[ch];
  float carry = 0.f, Ac = 1.f, Bc = 0.f;
  if (PASS == 2) {
    const int k0 = ck - idx;
    carry = p.cS[(size_t)k0 * W + ch];
    for (int k = k0; k < ck; k += 8) {
      float ca[8], cb[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const size_t o = (size_t)min(k + e, ck - 1) * W + ch;
        ca[e] = p.cA[o];
        cb[e] = p.cB[o];
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) carry = k + e < ck ? ca[e] * carry + cb[e] : carry;
    }
  }
  const int quads = bs / 4;
  T* ug = reinterpret_cast<T*>(p.u);
  for (int r0 = 0; r0 < (NT == 4 ? 1 : n); r0 += RT) {   // (NT = 4: a chunk is one tile)
    const int m = min(RT, n - r0);                   // (rows past the chunk repeat its last one; their steps are dropped)
    T yv[PASS == 2 ? NT : 1][4];
    if constexpr (PASS == 2) {
      const int oct = bs / 8;
      const T* yr = reinterpret_cast<const T*>(p.yx) + (size_t)(row0 + r0) * p.ld;
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          yv[t][i] = yr[(unsigned)(min(t * 16 + 4 * g + i, m - 1) * p.ld + ch)];
  #pragma unroll 1
    for (int x = tid; x < RT * oct; x += kScanWaves * 64) {
        const int i = x / oct, c = (x % oct) * 8;
        T* d = reinterpret_cast<T*>(us + i * stride) + c;
        const T* src = ug + (size_t)(row0 + r0 + min(i, m - 1)) * W + c0 + c;
#pragma unroll
        for (int e = 0; e < (int)sizeof(T) / 2; ++e) reinterpret_cast<uint4*>(d)[e] = reinterpret_cast<const uint4*>(src)[e];
      }
    } else {
  #pragma unroll 1
    for (int x = tid; x < RT / 4 * quads; x += kScanWaves * 64) {
        const int i0 = x / quads * 4, c = (x % quads) * 4, r = row0 + r0 + i0, last = row0 + r0 + m - 1;
        float u[4][4];
        if (r - run0 >= p.taps - 1) {
          conv_strip<T>(p, r, run0, last, c0 + c, u);
        } else {
#pragma unroll 1
          for (int i = 0; i < 4; ++i) {
            float v[4];
            conv4<T, 4>(p, min(r + i, last), min(r + i, last) - run0, st, pos0 <= 0, c0 + c, v);
            st4(reinterpret_cast<T*>(us + (i0 + i) * stride) + c, v);
            if (i0 + i < m && blockIdx.z == 0) st4(ug + (size_t)(r + i) * W + c0 + c, v);
          }
          continue;
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          st4(reinterpret_cast<T*>(us + (i0 + i) * stride) + c, u[i]);
          if (i0 + i < m && blockIdx.z == 0) st4(ug + (size_t)(r + i) * W + c0 + c, u[i]);
        }
      }
    }
    __builtin_amdgcn_sched_barrier(0);               // (the convolution's registers are free from here)
    f.load(gw, steps, 0);
    __syncthreads();
    if (active) {
      f32x4 ar[NT], ai[NT];
      gate_products<T, NT, PRE>(us, stride, gw, steps, f, ar, ai);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        float a[4], b[4], s[4], A, B;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int li = t * 16 + 4 * g + i;
          const float u = ldv(reinterpret_cast<const T*>(us + li * stride) + ct * 16 + rl);
          const Step q = lru_step(ar[t][i] + rb, ai[t][i] + ib, dec, u);
          a[i] = li < m ? q.a : 1.f;
          b[i] = li < m ? q.b : 0.f;
        }
        carry = scan_tile(a, b, carry, s, A, B);
        if (PASS == 1) {
          Bc = A * Bc + B;
          Ac = A * Ac;
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int li = t * 16 + 4 * g + i;
            if (li >= m) continue;
            const float y = gelu_tanh(ldv(&yv[t][i]) + yb);
            stv(reinterpret_cast<T*>(p.out) + (size_t)(row0 + r0) * p.ldo + (unsigned)(li * p.ldo + ch), s[i] * y);
          }
        }
        __builtin_amdgcn_sched_barrier(0);           // (one tile's registers at a time)
      }
    }
    __syncthreads();
  }
  if (active && g == 0) {
    if (PASS == 1) {
      p.cA[(size_t)ck * W + ch] = Ac;
      p.cB[(size_t)ck * W + ch] = Bc;
      if (idx == 0) p.cS[(size_t)ck * W + ch] = pos0 > 0 ? st[ch] : 0.f;
    } else if (idx == cnt - 1) {
      st[ch] = carry;
    }
  }
}

// the runs' last inputs (after the scan: its first chunks read the old ones)
template <class T>
__global__ __launch_bounds__(256) void rglru_inputs_kernel(RgLruParams p) {
  const int ck = blockIdx.y, ch = (blockIdx.x * 256 + threadIdx.x) * 4;
  const int row0 = p.chunks[4 * ck], n = p.chunks[4 * ck + 1], idx = p.chunks[4 * ck + 2], cnt = p.chunks[4 * ck + 3];
  if (idx != cnt - 1 || ch >= p.nb * p.bs) return;
  const int run0 = idx > 0 ? p.chunks[4 * (ck - idx)] : row0;
  save_inputs4<T>(p, row0 + n - 1, row0 + n - run0, p.positions[run0] == 0, p.state + (size_t)p.seq_ids[row0] * p.state_ld, ch);
}

int check(const RgLruParams& p) {
  if (p.rows < 1 || p.nb < 1 || p.bs < 32 || p.bs % 32 || p.taps < 1 || p.ld % 8 || p.state_ld % 4) return -1;
  if ((int64_t)p.ld < 2ll * p.nb * p.bs || p.ldo < p.nb * p.bs || p.state_ld < (int64_t)p.taps * p.nb * p.bs) return -2;
  if ((reinterpret_cast<uintptr_t>(p.yx) | reinterpret_cast<uintptr_t>(p.state) | reinterpret_cast<uintptr_t>(p.gw)) & 15) return -3;
  return 0;
}

template <class T>
size_t u_bytes(int rows, int bs) { return (size_t)rows * (bs * sizeof(T) + kPad); }

template <class T>
int launch_rows(const RgLruParams& p, hipStream_t st) {
  if (u_bytes<T>(16, p.bs) > kMaxLds) return -10;
  const dim3 grid(p.nb, (p.rows + 15) / 16), block(64 * (p.bs / 16 < 16 ? p.bs / 16 : 16));
  hipLaunchKernelGGL((rglru_rows_kernel<T>), grid, block, u_bytes<T>(16, p.bs), st, p);
  return (int)hipGetLastError();
}

template <class T, int NT>
int launch_scan_nt(const RgLruParams& p, hipStream_t st) {
  const dim3 grid(p.n_chunks, p.nb, (p.bs / 16 + kScanWaves - 1) / kScanWaves), block(kScanWaves * 64);
  const size_t lds = u_bytes<T>(16 * NT, p.bs);
  hipLaunchKernelGGL((rglru_scan_kernel<T, 1, NT>), grid, block, lds, st, p);
  hipLaunchKernelGGL((rglru_scan_kernel<T, 2, NT>), grid, block, lds, st, p);
  if (p.taps > 1)
    hipLaunchKernelGGL((rglru_inputs_kernel<T>), dim3((p.nb * p.bs / 4 + 255) / 256, p.n_chunks), dim3(256), 0, st, p);
  return (int)hipGetLastError();
}

template <class T>
int launch_scan(const RgLruParams& p, hipStream_t st) {
  if (u_bytes<T>(64, p.bs) <= 80 * 1024) return launch_scan_nt<T, 4>(p, st);
  if (u_bytes<T>(16, p.bs) <= kMaxLds) return launch_scan_nt<T, 1>(p, st);
  return -10;
}

}  // namespace

extern "C" int vwa_rglru_rows(const RgLruParams* p, hipStream_t st) {
  const int rc = check(*p);
  if (rc) return rc;
  if (p->rows > 64) return -4;
  return p->f32 ? launch_rows<float>(*p, st) : launch_rows<u16>(*p, st);
}

extern "C" int vwa_rglru_scan(const RgLruParams* p, hipStream_t st) {
  const int rc = check(*p);
  if (rc) return rc;
  if (p->n_chunks < 1 || !p->chunks || !p->cA || !p->cB || !p->cS || !p->u || (reinterpret_cast<uintptr_t>(p->u) & 15)) return -4;
  return p->f32 ? launch_scan<float>(*p, st) : launch_scan<u16>(*p, st);
}
