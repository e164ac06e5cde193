// Stubs of the launchers the core library leaves out (ops/build.py CORE): every call fails with a
// code the binding turns into an error.
#include "kernels/vwa_kernels.h"

namespace {
constexpr int kNotBuilt = -99;
}

extern "C" {
int vwa_skinny_gemm(int, const SkinnyParams*, hipStream_t) { return kNotBuilt; }
int vwa_chain_prepare(ChainParams*, int) { return kNotBuilt; }
int vwa_chain_launch(const ChainParams*, int, int, int, int, int, hipStream_t, int, int, int, int) { return kNotBuilt; }
int vwa_wdec_launch(const WdecParams*, int, hipStream_t) { return kNotBuilt; }
int vwa_decode_attention(const DecodeAttnParams*, hipStream_t) { return kNotBuilt; }
void vwa_set_attention_impl(int) {}
int vwa_flash_attention(const FlashAttnParams*, hipStream_t) { return kNotBuilt; }
int vwa_attention_split_tokens() { return 0; }
int vwa_pcm16_to_f32(const int16_t*, float*, int, int, float, hipStream_t) { return kNotBuilt; }
int vwa_log_mel(const float*, int, int, const float*, const float*, const float*, int, float*, float*, uint16_t*, int,
                hipStream_t) {
  return kNotBuilt;
}
void* vwa_ar_create(int, int, int64_t) { return nullptr; }
int vwa_ar_handles(void*, void*) { return kNotBuilt; }
int vwa_ar_handle_bytes() { return 0; }
int vwa_ar_open_peer(void*, int, const void*) { return kNotBuilt; }
int vwa_ar_allreduce(void*, const uint16_t*, uint16_t*, int64_t, hipStream_t) { return kNotBuilt; }
int vwa_ar_gather(void*, const int*, int*, int64_t, hipStream_t) { return kNotBuilt; }
int64_t vwa_ar_gather_max_words() { return 0; }
int vwa_ar_chain_tp(void*, ChainTP*) { return kNotBuilt; }
int vwa_ar_error(void*) { return kNotBuilt; }
void vwa_ar_destroy(void*) {}
}
