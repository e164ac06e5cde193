// Device parts of the gated recurrences, shared by their own launches (recurrence.hip) and the fused
// decode launch (stack_ops.hip).
#pragma once
#include "common.h"
#include "stack_kernels.h"
#include "stack_types.h"

namespace {
using namespace vwa;

struct Gate {
  float z, c;
};
VWA_DEVICE Gate min_gru_gate(float zp, float u) {
  return Gate{sigm(zp), u >= 0.f ? u + 0.5f : sigm(u)};
}

// Rows form of one (row, channel): the head row of a run of its sequence walks the run.
template <class T>
VWA_DEVICE void mingru_row(const MinGruParams& p, int r0, int ch) {
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

}  // namespace
