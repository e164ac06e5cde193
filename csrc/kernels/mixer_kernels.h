// Launch interface of the mixers and feed-forwards of serial layer stacks: the real-gated linear
// recurrence with its short convolution, latent attention, products per head or block, routed experts.
// Element type T of activations, caches and weights is bf16 (f32 = 0) or 32-bit float (f32 = 1).
//
// "Fragment order" of a weight W [N, K] (K a multiple of 4 EPL, EPL = 8 bf16 / 4 floats): for every
// 16-row tile and every 4 EPL deep step the 64 lanes' 16-byte MFMA operands,
// [N / 16][K / (4 EPL)][lane 16 g + n][e] = W[16 T + n][4 EPL step + EPL g + e].
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

// Recurrent block between its input and output projections.  Channels are padded block by block to a
// multiple of 32 (bs), width = nb * bs; padding channels have zero weights.
//   u_t = sum_k conv[k] (xp_(t - taps + 1 + k) + xb) + cb          (zeros before the sequence)
//   r, i = sigmoid(gate matrices of the block . u + bias);  a = exp(decay r)
//   S <- a S + sqrt(1 - a^2) i u;  out = S * gelu_tanh(yp + yb)
struct RgLruParams {
  const void* yx; int ld;           // [rows][y: width | x: width] T, the raw projections
  const float* yb; const float* xb; // [width]
  const float* cw; const float* cb; int taps;  // [taps][width] (last: the current token), [width]
  const void* gw;                   // T [nb][bs / 16][r, i][K = bs steps][64][EPL]: fragment order per block and gate
  const float* rb; const float* ib; // [width]
  const float* decay;               // [width]: -8 softplus(lam)
  int nb, bs, rows, f32;
  const int* seq_ids; const int* positions; const int64_t* slots;  // slot < 0: inert row (output zero, no state)
  float* state; int64_t state_ld;   // [state slots][taps * width]: S, then the last taps - 1 inputs (oldest first)
  void* out; int ldo;
  // scan form: chunks [n_chunks][4] = first row, rows (<= 64), index in its run, chunks of the run;
  // cA / cB / cS [n_chunks][width] f32 scratch, u [rows][width] T scratch
  const int* chunks; int n_chunks;
  float* cA; float* cB; float* cS;
  void* u;
};

// y[m][b * ys ..] = W_b . x[m][b * xs ..] for every head / block b (K inputs, N outputs)
struct HeadLinearParams {
  const int* row_list;              // rows of x and y this launch serves (null: 0 .. rows - 1)
  const void* x; int ldx; int xs;
  const void* w;                    // T fragment order per block [nb][N / 16][K steps][64][EPL]
  int nb, N, K, rows, f32;
  void* y; int ldy; int ys;
};

// Row part of latent attention: rotation of the heads' rotated query parts, norm of the latent, rotation
// of the shared key part, cache write ([latent: rank_p | rotated part: rot_p] per token).
struct LatentRowsParams {
  const void* x; int ldx;           // projected rows T: [q: H x (dim_p + rot_p) | latent rank_p | key part rot_p | ..]
  int rows, H, f32;
  int dim_p, rot_p, rot, rank, rank_p;
  const float* rope; int max_pos;   // [max_pos][rot / 2][cos, sin]
  const int* positions; const int64_t* slots;
  void* q_out; int ldq; int q_head; int q_at;  // head h's rotated part goes to column h * q_head + q_at
  int has_kv;                       // 0: the layer reads another layer's cache
  const float* norm; float eps;     // [rank]
  void* cache; int64_t c_sb; int block_size;   // [blocks][block_size][rank_p + rot_p]
};

// Causal attention of ragged rows over cached latents, queries already in latent space:
// q row = H x [rank_p | rot_p].  Writes unnormalised partial sums per key chunk; merged (with the sinks)
// by vwa_latent_out.
struct LatentAttnParams {
  const void* q; int ldq;
  const void* cache; int64_t c_sb; const int* block_table; int table_stride, block_size;
  const int* positions; const int* seq_ids; const int64_t* slots;
  const int* row_list;              // rows this launch serves (null: 0 .. rows - 1)
  int rows, H, rank_p, rot_p, f32;
  float scale;
  int nch;                          // key chunks per row
  float* part;                      // [rows][nch][H][rank_p]
  float* stat;                      // [rows][nch][H][2] (max, sum); sum 0: no key in the chunk
};

// Merge of the chunks with the sinks, value projection and output gate:
// out[row][h * vd ..] = sigmoid(gate) * W_h . (latent sum of head h)
struct LatentOutParams {
  const float* part; const float* stat; int nch;
  const int64_t* slots; const int* row_list;
  int rows, H, rank_p, vd, f32;
  const float* sink;                // [H]
  const void* w;                    // T fragment order per head [H][vd / 16][rank_p steps][64][EPL]
  const void* gate; int ldg;        // [.., H * vd]
  void* out; int ldo;
};

// Latent attention of prompt-sized runs (bf16) over expanded keys and values (latent_prefill.hip).
// gather: segs [n_segs][3] = block-table row, first key, keys of its run -- 64 rows of lat / krot each;
// prefill: q_tiles [n_tiles][4] = first row, rows (<= 128), row of the run's key 0 in kv / krot, position of the
// first row.  kv rows: [keys H x dim_p | values H x vdk]; runs' contexts are padded to 64 rows.
struct LatentPrefillParams {
  const void* cache; int64_t c_sb; const int* block_table; int table_stride, block_size;
  const int* segs; int n_segs;
  int rank_p, rot_p, kp;
  uint16_t* lat; uint16_t* krot;    // [64 n_segs][kp], [64 n_segs][rot_p]
  const int* q_tiles; int n_tiles;
  int H, dim_p, vdk, vd;            // value columns in kv (a multiple of 32) and in out / gate
  float scale;
  const void* qn; int ldqn;         // projected rows, head h at h * (dim_p + rot_p)
  const void* qr; int ldqr; int qr_head, qr_at;   // rotated parts
  const void* kv; int ldkv;
  const float* sink;
  const void* gate; int ldg;
  void* out; int ldo;
};

// Routed experts.  A pair is (row, k): row's k-th choice, pair id = row * top + k.
struct MoeRouteParams {
  const void* h; int ldh; int K;    // [rows, K] T (K a multiple of the fragment step)
  const void* w;                    // router in fragment order [E_p / 16][K steps][64][EPL]
  int rows, E, top, f32;
  const int64_t* slots;             // rows with slot < 0 choose nothing
  float* wts; int* ids;             // [rows * top]: score and expert of every pair (inert: -1)
  int tile;                         // pairs per tile (16, 32, 128 or 256)
  int max_tiles;
  int* tiles;                       // [1 + 3 * max_tiles]: count, then (expert, first sorted place, pairs)
  int* order;                       // [max_tiles * tile]: sorted place -> pair
  int* ticket;                      // zero between launches
};
// act[place] = silu(w g) * (w u), g / u = W_gate / W_up of the tile's expert . h[row of the pair]  (down = 0)
// y[pair] = W_down of the expert . act[place]                                                       (down = 1)
struct MoeGemmParams {
  const void* x; int ldx;
  const void* w; int64_t w_expert;  // elements per expert; pre-tiled order (ops.mixers.tile_weight)
  int N, K, top, f32, down;         // N: rows of one expert's matrix (gate / up interleaved by 16: 2 x ff)
  const float* wts;
  const int* tiles; const int* order; int max_tiles, tile;   // tile: 16, 32, or 128 / 256 (bf16: the LDS-tiled GEMM)
  int x_rows;                       // rows of x
  void* y; int ldy;
};

#ifdef __cplusplus
extern "C" {
#endif
int vwa_rglru_rows(const RgLruParams* p, hipStream_t st);
int vwa_rglru_scan(const RgLruParams* p, hipStream_t st);
int vwa_head_linear(const HeadLinearParams* p, hipStream_t st);
int vwa_latent_rows(const LatentRowsParams* p, hipStream_t st);
// a decode step's rows: latent_rows and the queries' product with the key projection in one launch
int vwa_latent_qkv(const LatentRowsParams* p, const HeadLinearParams* q, hipStream_t st);
int vwa_latent_attention(const LatentAttnParams* p, hipStream_t st);
int vwa_latent_out(const LatentOutParams* p, hipStream_t st);
int vwa_latent_prefill_fits(int dim_p, int rot_p, int vdk);
int vwa_latent_gather(const LatentPrefillParams* p, hipStream_t st);
int vwa_latent_prefill(const LatentPrefillParams* p, hipStream_t st);
int vwa_moe_route(const MoeRouteParams* p, hipStream_t st);
int vwa_moe_gemm(const MoeGemmParams* p, hipStream_t st);
// x (f32 rows) += norm(sum of the row's n_parts branch rows) * w1; h (T) = norm(x) * w2 (w2 null: no h)
int vwa_add_norm(float* x, int ldx, const void* br, int ldb, int n_parts, const float* w1, const float* w2, void* h, int ldh,
                 int rows, int D, int Dpad, float eps, int f32, hipStream_t st);
#ifdef __cplusplus
}
#endif
