// Launch interface of the kernels for layer stacks with an f32 residual stream: norms, partial
// rotation + cache write, windowed attention with mixed heads, gated recurrences, 32-bit GEMM.
// Element type T of activations, caches and weights is bf16 (f32 = 0) or 32-bit float (f32 = 1).
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

// Y[M, N] = epi(X[M, K] . W[N, K]^T) in 32-bit (f32 MFMA).  epi as gemm.hip: 0 store, 1 residual add,
// 2 SwiGLU over gate / up rows interleaved per 16 (Y [M, N / 2]), 6 split (columns >= n_split: relu(v)^2 -> Y2)
struct GemmF32Params {
  const float* X; int ldx;
  const float* W;                   // row-major [N, K]
  int M, N, K;
  float* Y; int ldy;
  const float* R; int ldr;
  int n_split; float* Y2; int ldy2;
};

// Rotation of the first rot_dims dimensions of every q / k head (pairs (i, i + rot_dims / 2), table
// [max_pos][rot_dims / 2][cos, sin]) and the cache write of one step's rows:
//   x row = [q: H heads x dk | k: G x dk | v: G x dv] (T)
//   q -> q_out [rows, H * dk]; k -> K cache [blocks][G][block_size][dk];
//   v -> V cache, TRANSPOSED inside a block: [blocks][G][dv][block_size] -- the order in which the
//   MFMA takes V^T as its A operand, so attention reads it without staging
struct QkvCacheParams {
  const void* x; int ldx;
  int rows, H, G, dk, dv, rot_dims, f32;
  const float* rope; int max_pos;
  const int* positions; const int64_t* slots;   // slot < 0: row without a cache entry
  void* q_out; int ldq;
  void* k; void* v; int64_t k_sb, k_sh, v_sb, v_sh; int block_size;
};

// Attention over the visible keys of each row (j <= i and (i - j < window or j < keep); window 0: all)
// with the heads' softmax weights mixed across heads (talk [H][H]; null: not mixed), an optional
// per-head output gate sigmoid(gate[row][h]) and a constant output scale.
// Keys are walked in 16-key tiles (a tile never crosses a cache block), dealt to workgroups in chunks of at most 8.
struct TalkAttnParams {
  const void* q; int ldq;           // [rows, H * dk]
  const void* k; const void* v; int64_t k_sb, k_sh, v_sb, v_sh;
  const int* block_table; int table_stride, block_size;
  const int* positions; const int* seq_ids; const int64_t* slots;
  const int* row_list;              // rows this launch serves (null: 0 .. rows - 1)
  int rows, H, G, dk, dv, f32;
  float scale; int window, keep;
  const float* talk;
  const void* gate; int ldg;        // [.., H] pre-activations (T) or null
  float out_scale;
  int nch;                          // chunks per row the scratch holds
  float* s;                         // [rows][H][nch * 128] scores
  float* stat;                      // [rows][H][nch][2] (max, sum) per chunk
  float* part;                      // [rows][nch][H][dv] partial outputs
  int* counters;                    // [rows * G * ceil(H / G / 16)] chunk tickets, zero between launches
  void* out; int ldo;               // [.., H * dv] T
};

// The same attention for runs of consecutive prompt rows (bf16): one workgroup per 16 queries
struct TalkPrefillParams {
  TalkAttnParams a;                 // (row_list / nch / s / stat / part / counters unused)
  const int* tiles;                 // [n_tiles][2]: first row, rows (1..16) -- one sequence, consecutive positions
  int n_tiles;
  // talk (identity if not mixed) as the MFMA A operand over the padded heads h = c * RP + r (kv heads GP
  // and query heads per kv head RP rounded up to powers of two, HT = GP * RP): bf16 [HT > 16 ? 2 : 1]
  // [64 lanes][8], lane (row rl, group b), element e: talk[16 mt + rl][head of k], k = 8 b + e -- HT 32:
  // head k; 16: k mod 16; 8: k mod 8 for k < 16, else 0; <= 4: k mod 4 for k < 8, else 0
  const uint16_t* talk_frag;
  int max_tiles;                    // key tiles a query tile can see at most (<= 1024)
  float* lse;                       // [rows of q][H] scratch
  int splits;                       // workgroups per tile over its keys
  float* part;                      // [n_tiles][splits][vwa_talk_prefill_part floats] (splits > 1)
  int* tickets;                     // [n_tiles], zero between launches (splits > 1)
};

// Gated recurrence of one layer over a step's rows: z = sigmoid(zp + zb), u = xp + xb,
// S <- (1 - z) S + z (u >= 0 ? u + 1/2 : sigmoid(u)); out = S * silu(gp) * out_scale.  f32 state.
struct MinGruParams {
  const void* z; const void* x; const void* g; int ld;   // projections [rows, width] T
  const float* zb; const float* xb;
  const int* seq_ids; const int* positions; const int64_t* slots;
  int rows, width, f32;
  float* state; int state_ld;       // [state slots][width]; the slot is the row's sequence id
  float out_scale;
  void* out; int ldo;
  // chunked scan (prompt-sized runs): chunks [n_chunks][4] = first row, rows, index in its run, chunks
  // of the run; A / B / S0: [n_chunks][width] f32 scratch
  const int* chunks; int n_chunks;
  float* cA; float* cB; float* cS;
};

#ifdef __cplusplus
extern "C" {
#endif
int vwa_gemm_f32(int epi, const GemmF32Params* p, hipStream_t st);
// y (T) [rows, ldy] = layer norm of x f32 rows over D columns (b null: no bias); columns D .. Dpad-1 of y are zeroed
int vwa_layernorm_f32(const float* x, int ldx, const float* w, const float* b, void* y, int ldy, int rows, int D, int Dpad,
                      float eps, int f32, hipStream_t st);
// out f32 [rows, ldo] = table (T) rows * scale; ids outside the table give zeros; columns D .. Dpad-1 are zeroed
int vwa_embedding_f32(const int* ids, const void* table, int ld, float* out, int ldo, int rows, int D, int Dpad, int vocab,
                      float scale, int f32, hipStream_t st);
int vwa_qkv_cache(const QkvCacheParams* p, hipStream_t st);
// a decode step's qkv_cache and mingru_rows over the same rows, one launch
int vwa_qkv_mingru(const QkvCacheParams* p, const MinGruParams* g, hipStream_t st);
int vwa_talk_attention(const TalkAttnParams* p, hipStream_t st);
int vwa_talk_prefill(const TalkPrefillParams* p, hipStream_t st);
// partial floats per (tile, split) of vwa_talk_prefill, < 0 if it does not take these sizes
int64_t vwa_talk_prefill_part(int H, int G, int dk, int dv);
int vwa_mingru_rows(const MinGruParams* p, hipStream_t st);
int vwa_mingru_scan(const MinGruParams* p, hipStream_t st);
#ifdef __cplusplus
}
#endif
