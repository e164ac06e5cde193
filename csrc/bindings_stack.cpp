// Torch bindings of the layer-stack kernels (stack_kernels.h): f32 residual rows, T = bf16 or f32
// activations / caches / weights.  Shapes, dtypes and strides are checked here, before any launch.
#include "bindings_checks.h"
#include "kernels/mixer_kernels.h"
#include "kernels/stack_kernels.h"

namespace {

void gemm_f32(Tensor x, Tensor w, Tensor y, int64_t epi, c10::optional<Tensor> residual, c10::optional<Tensor> y2) {
  c10::DeviceGuard g(x.device());
  check_t(x, true, "x");
  check_t(w, true, "w");
  check_t(y, true, "y");
  TORCH_CHECK(w.dim() == 2 && w.is_contiguous(), "w must be contiguous [N, K]");
  const int64_t M = x.size(0), N = w.size(0), K = w.size(1);
  TORCH_CHECK(x.dim() == 2 && x.stride(1) == 1 && x.size(1) == K, "x must be [M, K]");
  TORCH_CHECK(K % 16 == 0 && x.stride(0) % 4 == 0, "gemm_f32: K % 16 == 0, 16-byte aligned rows");
  check_aligned(x, "x");
  check_aligned(w, "w");
  GemmF32Params p{};
  p.X = x.data_ptr<float>();
  p.ldx = (int)x.stride(0);
  p.W = w.data_ptr<float>();
  p.M = (int)M;
  p.N = (int)N;
  p.K = (int)K;
  TORCH_CHECK(y.dim() == 2 && y.size(0) == M, "y rows");
  p.Y = y.data_ptr<float>();
  p.ldy = (int)y.stride(0);
  if (epi == 2) {
    TORCH_CHECK(N % 32 == 0 && y.size(1) * 2 == N && y.stride(1) == 1, "SwiGLU epilogue: y [M, N / 2], N a multiple of 32");
  } else if (epi == 6) {
    TORCH_CHECK(y2.has_value(), "split epilogue needs y2");
    check_t(*y2, true, "y2");
    check_rows(*y2, M, 1, "y2");
    TORCH_CHECK(y.size(1) + y2->size(1) == N && y.stride(1) == 1, "split epilogue: y and y2 columns must add up to N");
    p.Y2 = y2->data_ptr<float>();
    p.ldy2 = (int)y2->stride(0);
    p.n_split = (int)y.size(1);
  } else {
    TORCH_CHECK(y.size(1) == N && y.stride(1) == 1, "y columns");
  }
  if (epi == 1) {
    TORCH_CHECK(residual.has_value(), "residual epilogue needs residual");
    check_t(*residual, true, "residual");
    check_rows(*residual, M, N, "residual");
    p.R = residual->data_ptr<float>();
    p.ldr = (int)residual->stride(0);
  }
  check_rc(vwa_gemm_f32((int)epi, &p, cur_stream(x)), "gemm_f32");
}

void layernorm_f32(Tensor x, Tensor w, c10::optional<Tensor> b, Tensor y, double eps) {
  c10::DeviceGuard g(x.device());
  check_t(x, true, "x");
  const bool f32 = t_is_f32(y, "y");
  const int64_t D = w.numel(), rows = y.size(0);
  f32p(w, D, "w");
  check_rows(x, rows, D, "x");
  check_rows(y, rows, D, "y");
  check_aligned(x, "x");
  check_aligned(y, "y");
  check_rc(vwa_layernorm_f32(x.data_ptr<float>(), (int)x.stride(0), w.data_ptr<float>(),
                             b.has_value() ? f32p(*b, D, "b") : nullptr, y.data_ptr(),
                             (int)y.stride(0), (int)rows, (int)D, (int)y.size(1), (float)eps, f32, cur_stream(x)),
           "layernorm_f32");
}

// x (f32 rows) += norm(sum of the row's n_parts branch rows) * w1; h = norm(x) * w2 (no w2: no h)
void add_norm(Tensor x, Tensor br, int64_t n_parts, Tensor w1, c10::optional<Tensor> w2, c10::optional<Tensor> h, double eps) {
  c10::DeviceGuard g(x.device());
  check_t(x, true, "x");
  const bool f32 = t_is_f32(br, "branch");
  const int64_t D = w1.numel(), rows = x.size(0), q = (D + 3) / 4 * 4;
  TORCH_CHECK(n_parts >= 1, "n_parts");
  check_rows(x, rows, q, "x");
  check_rows(br, rows * n_parts, q, "branch");
  check_aligned(x, "x");
  check_aligned(br, "branch");
  const float* p1 = f32p(w1, D, "w1");
  const float* p2 = w2.has_value() ? f32p(*w2, D, "w2") : nullptr;
  if (p2) {
    TORCH_CHECK(h.has_value(), "w2 needs h");
    check_t(*h, f32, "h");
    check_rows(*h, rows, q, "h");
    check_aligned(*h, "h");
  }
  check_rc(vwa_add_norm(x.data_ptr<float>(), (int)x.stride(0), br.data_ptr(), (int)br.stride(0), (int)n_parts, p1, p2,
                        p2 ? h->data_ptr() : nullptr, p2 ? (int)h->stride(0) : 0, (int)rows, (int)D, p2 ? (int)h->size(1) : 0,
                        (float)eps, f32, cur_stream(x)),
           "add_norm");
}

void embedding_f32(Tensor ids, Tensor table, Tensor out, double scale) {
  c10::DeviceGuard g(out.device());
  const bool f32 = t_is_f32(table, "table");
  check_t(out, true, "out");
  TORCH_CHECK(table.dim() == 2 && table.stride(1) == 1, "table [vocab, D]");
  const int64_t rows = out.size(0);
  check_rows(out, rows, table.size(1), "out");
  check_rc(vwa_embedding_f32(i32p(ids, rows, "ids"), table.data_ptr(), (int)table.stride(0), out.data_ptr<float>(),
                             (int)out.stride(0), (int)rows, (int)table.size(1), (int)out.size(1), (int)table.size(0),
                             (float)scale, f32, cur_stream(out)),
           "embedding_f32");
}

// K [blocks, G, block_size, dk] and V [blocks, G, dv, block_size], contiguous inside a kv head
void check_caches(const Tensor& k, const Tensor& v, bool f32, int64_t G, int64_t dk, int64_t dv) {
  check_t(k, f32, "k cache");
  check_t(v, f32, "v cache");
  TORCH_CHECK(k.dim() == 4 && v.dim() == 4 && k.size(0) == v.size(0) && k.size(1) == G && v.size(1) == G && k.size(3) == dk &&
                  v.size(2) == dv && v.size(3) == k.size(2),
              "k cache [blocks, ", G, ", block_size, ", dk, "], v cache [blocks, ", G, ", ", dv, ", block_size]");
  TORCH_CHECK(k.stride(3) == 1 && k.stride(2) == dk && v.stride(3) == 1 && v.stride(2) == v.size(3),
              "caches must be contiguous inside a kv head");
  check_aligned(k, "k cache");
  check_aligned(v, "v cache");
}

QkvCacheParams qkv_params(const Tensor& x, int64_t H, int64_t G, int64_t dk, int64_t dv, int64_t rot_dims, const Tensor& rope,
                          const Tensor& positions, const Tensor& slots, const Tensor& q_out, const Tensor& k, const Tensor& v) {
  const bool f32 = t_is_f32(x, "x");
  const int64_t rows = q_out.size(0);
  check_rows(x, rows, H * dk + G * (dk + dv), "x");
  check_t(q_out, f32, "q_out");
  check_rows(q_out, rows, H * dk, "q_out");
  check_aligned(x, "x");
  check_aligned(q_out, "q_out");
  check_caches(k, v, f32, G, dk, dv);
  TORCH_CHECK(rope.is_cuda() && rope.scalar_type() == at::kFloat && rope.is_contiguous() && rope.dim() == 3 && rope.size(0) >= 1 &&
                  rope.size(1) * 2 == rot_dims && rope.size(2) == 2,
              "rope table f32 [max_pos, rot_dims / 2, 2]");
  QkvCacheParams p{};
  p.x = x.data_ptr();
  p.ldx = (int)x.stride(0);
  p.rows = (int)rows;
  p.H = (int)H;
  p.G = (int)G;
  p.dk = (int)dk;
  p.dv = (int)dv;
  p.rot_dims = (int)rot_dims;
  p.f32 = f32;
  p.rope = rope.data_ptr<float>();
  p.max_pos = (int)rope.size(0);
  p.positions = i32p(positions, rows, "positions");
  p.slots = i64p(slots, rows, "slots");
  p.q_out = q_out.data_ptr();
  p.ldq = (int)q_out.stride(0);
  p.k = k.data_ptr();
  p.v = v.data_ptr();
  p.k_sb = k.stride(0);
  p.k_sh = k.stride(1);
  p.v_sb = v.stride(0);
  p.v_sh = v.stride(1);
  p.block_size = (int)k.size(2);
  return p;
}

void qkv_cache(Tensor x, int64_t H, int64_t G, int64_t dk, int64_t dv, int64_t rot_dims, Tensor rope, Tensor positions,
               Tensor slots, Tensor q_out, Tensor k, Tensor v) {
  c10::DeviceGuard g(x.device());
  const QkvCacheParams p = qkv_params(x, H, G, dk, dv, rot_dims, rope, positions, slots, q_out, k, v);
  check_rc(vwa_qkv_cache(&p, cur_stream(x)), "qkv_cache");
}

TalkAttnParams attn_params(const Tensor& q, const Tensor& k, const Tensor& v, const Tensor& table, const Tensor& positions,
                           const Tensor& seq_ids, const Tensor& slots, int64_t n_rows, int64_t H, double scale, int64_t window,
                           int64_t keep, const c10::optional<Tensor>& talk, const c10::optional<Tensor>& gate, double out_scale,
                           const Tensor& out) {
  TalkAttnParams p{};
  const bool f32 = t_is_f32(q, "q");
  TORCH_CHECK(k.dim() == 4 && v.dim() == 4, "caches must be 4-D");
  const int64_t G = k.size(1), dk = k.size(3), dv = v.size(2);
  check_caches(k, v, f32, G, dk, dv);
  TORCH_CHECK(H >= 1 && H % G == 0, "query heads must be a multiple of the kv heads");
  check_rows(q, n_rows, H * dk, "q");
  check_t(out, f32, "out");
  check_rows(out, n_rows, H * dv, "out");
  check_aligned(q, "q");
  TORCH_CHECK(q.stride(0) % 8 == 0, "q rows must be 16-byte aligned");
  TORCH_CHECK(table.is_cuda() && table.scalar_type() == at::kInt && table.dim() == 2 && table.stride(1) == 1, "block table int32");
  p.q = q.data_ptr();
  p.ldq = (int)q.stride(0);
  p.k = k.data_ptr();
  p.v = v.data_ptr();
  p.k_sb = k.stride(0);
  p.k_sh = k.stride(1);
  p.v_sb = v.stride(0);
  p.v_sh = v.stride(1);
  p.block_table = table.data_ptr<int>();
  p.table_stride = (int)table.stride(0);
  p.block_size = (int)k.size(2);
  p.positions = i32p(positions, n_rows, "positions");
  p.seq_ids = i32p(seq_ids, n_rows, "seq_ids");
  p.slots = i64p(slots, n_rows, "slots");
  p.H = (int)H;
  p.G = (int)G;
  p.dk = (int)dk;
  p.dv = (int)dv;
  p.f32 = f32;
  p.scale = (float)scale;
  p.window = (int)window;
  p.keep = (int)keep;
  if (talk.has_value()) p.talk = f32p(*talk, H * H, "talk");
  if (gate.has_value()) {
    check_t(*gate, f32, "gate");
    check_rows(*gate, n_rows, H, "gate");
    p.gate = gate->data_ptr();
    p.ldg = (int)gate->stride(0);
  }
  p.out_scale = (float)out_scale;
  p.out = out.data_ptr();
  p.ldo = (int)out.stride(0);
  return p;
}

// Tiles of 16 keys a row can see at most: the kept ones plus the window's (or the whole context)
int64_t max_tiles(int64_t max_ctx, int64_t window, int64_t keep) {
  const int64_t all = (max_ctx + 15) / 16;
  if (window <= 0) return all;
  return std::min(all, (keep + 15) / 16 + (window + 14) / 16 + 1);
}

void talk_attention(Tensor q, Tensor k, Tensor v, Tensor table, Tensor positions, Tensor seq_ids, Tensor slots,
                    c10::optional<Tensor> row_list, int64_t n_rows, int64_t H, double scale, int64_t window, int64_t keep,
                    c10::optional<Tensor> talk, c10::optional<Tensor> gate, double out_scale, int64_t max_ctx, Tensor s,
                    Tensor stat, Tensor part, Tensor counters, Tensor out) {
  c10::DeviceGuard g(q.device());
  const int64_t total = q.size(0);
  TalkAttnParams p = attn_params(q, k, v, table, positions, seq_ids, slots, row_list.has_value() ? total : n_rows, H, scale,
                                 window, keep, talk, gate, out_scale, out);
  TORCH_CHECK(max_ctx >= 1 && max_ctx <= table.size(1) * k.size(2), "max_ctx exceeds the block table");
  if (row_list.has_value()) p.row_list = i32p(*row_list, n_rows, "row_list");
  p.rows = (int)n_rows;
  const int64_t nch = (max_tiles(max_ctx, window, keep) + 7) / 8, R = H / p.G;
  p.nch = (int)nch;
  p.s = f32p(s, n_rows * H * nch * 128, "s");
  p.stat = f32p(stat, n_rows * H * nch * 2, "stat");
  p.part = f32p(part, n_rows * nch * H * p.dv, "part");
  i32p(counters, n_rows * p.G * ((R + 15) / 16), "counters");
  p.counters = counters.data_ptr<int>();
  check_rc(vwa_talk_attention(&p, cur_stream(q)), "talk_attention");
}

void talk_prefill(Tensor q, Tensor k, Tensor v, Tensor table, Tensor positions, Tensor seq_ids, Tensor slots, Tensor tiles,
                  int64_t H, double scale, int64_t window, int64_t keep, Tensor talk_frag, c10::optional<Tensor> gate,
                  double out_scale, int64_t max_ctx, int64_t splits, Tensor lse, Tensor part, Tensor tickets, Tensor out) {
  c10::DeviceGuard g(q.device());
  TalkPrefillParams p{};
  p.a = attn_params(q, k, v, table, positions, seq_ids, slots, q.size(0), H, scale, window, keep, c10::nullopt, gate, out_scale,
                    out);
  TORCH_CHECK(max_ctx >= 1 && max_ctx <= table.size(1) * k.size(2), "max_ctx exceeds the block table");
  p.a.rows = (int)q.size(0);
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2 && tiles.size(0) >= 1, "tiles int32 [n, 2]");
  p.tiles = i32p(tiles, tiles.numel(), "tiles");
  p.n_tiles = (int)tiles.size(0);
  TORCH_CHECK(talk_frag.is_cuda() && talk_frag.scalar_type() == at::kBFloat16 && talk_frag.is_contiguous() &&
                  talk_frag.numel() >= (H > 16 ? 1024 : 512),
              "talk_frag bf16 [tiles, 64, 8] (ops.talk_fragment)");
  check_aligned(talk_frag, "talk_frag");
  p.talk_frag = bfp(talk_frag);
  p.max_tiles = (int)max_tiles(max_ctx, window > 0 ? window + 15 : 0, keep);
  p.lse = f32p(lse, q.size(0) * H, "lse");
  p.splits = (int)splits;
  if (splits > 1) {
    const int64_t per = vwa_talk_prefill_part((int)H, p.a.G, p.a.dk, p.a.dv);
    TORCH_CHECK(per > 0, "talk_prefill does not take these sizes");
    p.part = f32p(part, p.n_tiles * splits * per, "part");
    check_aligned(part, "part");
    i32p(tickets, p.n_tiles, "tickets");
    p.tickets = tickets.data_ptr<int>();
  }
  TORCH_CHECK((reinterpret_cast<uintptr_t>(out.data_ptr()) & 7) == 0, "out rows must be 8-byte aligned");
  check_rc(vwa_talk_prefill(&p, cur_stream(q)), "talk_prefill");
}

MinGruParams mingru_params(const Tensor& z, const Tensor& x, const Tensor& gt, const c10::optional<Tensor>& zb,
                           const c10::optional<Tensor>& xb, const Tensor& seq_ids, const Tensor& positions, const Tensor& slots,
                           const Tensor& state, double out_scale, const Tensor& out) {
  const bool f32 = t_is_f32(z, "z");
  const int64_t rows = out.size(0), width = state.size(1);
  for (const Tensor* t : {&z, &x, &gt}) {
    check_t(*t, f32, "projection");
    check_rows(*t, rows, width, "projection");
    TORCH_CHECK(t->stride(0) == z.stride(0), "projections must share one row stride");
  }
  check_t(out, f32, "out");
  check_rows(out, rows, width, "out");
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.dim() == 2 && state.is_contiguous(), "state f32 [slots, width]");
  MinGruParams p{};
  p.z = z.data_ptr();
  p.x = x.data_ptr();
  p.g = gt.data_ptr();
  p.ld = (int)z.stride(0);
  if (zb.has_value()) p.zb = f32p(*zb, width, "zb");
  if (xb.has_value()) p.xb = f32p(*xb, width, "xb");
  p.seq_ids = i32p(seq_ids, rows, "seq_ids");
  p.positions = i32p(positions, rows, "positions");
  p.slots = i64p(slots, rows, "slots");
  p.rows = (int)rows;
  p.width = (int)width;
  p.f32 = f32;
  p.state = state.data_ptr<float>();
  p.state_ld = (int)state.stride(0);
  p.out_scale = (float)out_scale;
  p.out = out.data_ptr();
  p.ldo = (int)out.stride(0);
  return p;
}

void mingru(Tensor z, Tensor x, Tensor gt, c10::optional<Tensor> zb, c10::optional<Tensor> xb, Tensor seq_ids, Tensor positions,
            Tensor slots, Tensor state, double out_scale, Tensor out, c10::optional<Tensor> chunks, c10::optional<Tensor> scratch) {
  c10::DeviceGuard g(z.device());
  MinGruParams p = mingru_params(z, x, gt, zb, xb, seq_ids, positions, slots, state, out_scale, out);
  const int64_t width = p.width;
  if (!chunks.has_value()) {
    check_rc(vwa_mingru_rows(&p, cur_stream(z)), "mingru_rows");
    return;
  }
  TORCH_CHECK(chunks->dim() == 2 && chunks->size(1) == 4 && chunks->size(0) >= 1, "chunks int32 [n, 4]");
  p.chunks = i32p(*chunks, chunks->numel(), "chunks");
  p.n_chunks = (int)chunks->size(0);
  TORCH_CHECK(scratch.has_value(), "scan form needs scratch");
  float* s = f32p(*scratch, 3 * (int64_t)p.n_chunks * width, "scratch");
  p.cA = s;
  p.cB = s + (size_t)p.n_chunks * width;
  p.cS = s + (size_t)2 * p.n_chunks * width;
  check_rc(vwa_mingru_scan(&p, cur_stream(z)), "mingru_scan");
}

// a decode step's rows: rotation + cache write and the recurrence in one launch (arguments of both)
void qkv_mingru(Tensor x, int64_t H, int64_t G, int64_t dk, int64_t dv, int64_t rot_dims, Tensor rope, Tensor positions,
                Tensor slots, Tensor q_out, Tensor k, Tensor v, Tensor z, Tensor u, Tensor gt, c10::optional<Tensor> zb,
                c10::optional<Tensor> xb, Tensor seq_ids, Tensor state, double out_scale, Tensor out) {
  c10::DeviceGuard g(x.device());
  const QkvCacheParams p = qkv_params(x, H, G, dk, dv, rot_dims, rope, positions, slots, q_out, k, v);
  const MinGruParams m = mingru_params(z, u, gt, zb, xb, seq_ids, positions, slots, state, out_scale, out);
  check_rc(vwa_qkv_mingru(&p, &m, cur_stream(x)), "qkv_mingru");
}

}  // namespace

void bind_stack(py::module_& m) {
  m.def("gemm_f32", &gemm_f32, py::arg("x"), py::arg("w"), py::arg("y"), py::arg("epi"), py::arg("residual") = py::none(),
        py::arg("y2") = py::none());
  m.def("layernorm_f32", &layernorm_f32);
  m.def("add_norm", &add_norm);
  m.def("embedding_f32", &embedding_f32);
  m.def("qkv_cache", &qkv_cache);
  m.def("qkv_mingru", &qkv_mingru);
  m.def("talk_prefill_part", [](int64_t H, int64_t G, int64_t dk, int64_t dv) {
    return vwa_talk_prefill_part((int)H, (int)G, (int)dk, (int)dv);
  });
  m.def("talk_attention", &talk_attention, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("positions"),
        py::arg("seq_ids"), py::arg("slots"), py::arg("row_list"), py::arg("n_rows"), py::arg("H"), py::arg("scale"),
        py::arg("window"), py::arg("keep"), py::arg("talk"), py::arg("gate"), py::arg("out_scale"), py::arg("max_ctx"),
        py::arg("s"), py::arg("stat"), py::arg("part"), py::arg("counters"), py::arg("out"));
  m.def("talk_prefill", &talk_prefill, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("table"), py::arg("positions"),
        py::arg("seq_ids"), py::arg("slots"), py::arg("tiles"), py::arg("H"), py::arg("scale"), py::arg("window"),
        py::arg("keep"), py::arg("talk_frag"), py::arg("gate"), py::arg("out_scale"), py::arg("max_ctx"), py::arg("splits"),
        py::arg("lse"), py::arg("part"), py::arg("tickets"), py::arg("out"));
  m.def("mingru", &mingru, py::arg("z"), py::arg("x"), py::arg("g"), py::arg("zb"), py::arg("xb"), py::arg("seq_ids"),
        py::arg("positions"), py::arg("slots"), py::arg("state"), py::arg("out_scale"), py::arg("out"),
        py::arg("chunks") = py::none(), py::arg("scratch") = py::none());
}
