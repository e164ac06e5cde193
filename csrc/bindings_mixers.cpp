// Torch bindings of the serial-stack mixers and feed-forwards (mixer_kernels.h).
#include "bindings_checks.h"
#include "kernels/mixer_kernels.h"

namespace {

using OptTensor = c10::optional<Tensor>;

const void* frag(const Tensor& w, bool f32, int64_t n, const char* name) {
  check_t(w, f32, name);
  TORCH_CHECK(w.is_contiguous() && w.numel() == n, name, ": ", n, " elements in fragment order, got ", w.numel());
  check_aligned(w, name);
  return w.data_ptr();
}

// y | x projections [rows, 2 width]; conv [taps, width]; state [slots, taps * width]; chunks / scratch: scan form
void rglru(Tensor yx, Tensor yb, Tensor xb, Tensor cw, Tensor cb, Tensor gw, Tensor rb, Tensor ib, Tensor decay, int64_t nb,
           Tensor seq_ids, Tensor positions, Tensor slots, Tensor state, Tensor out, OptTensor chunks, OptTensor scratch,
           OptTensor u) {
  c10::DeviceGuard g(yx.device());
  const bool f32 = t_is_f32(yx, "yx");
  const int64_t rows = out.size(0), W = decay.numel();
  TORCH_CHECK(nb >= 1 && W % nb == 0 && (W / nb) % 32 == 0, "blocks of a multiple of 32 channels");
  const int64_t bs = W / nb;
  check_rows(yx, rows, 2 * W, "yx");
  check_aligned(yx, "yx");
  TORCH_CHECK(yx.stride(0) % 8 == 0, "yx rows must be 16-byte aligned");
  check_t(out, f32, "out");
  check_rows(out, rows, W, "out");
  TORCH_CHECK(cw.dim() == 2 && cw.size(0) >= 1 && cw.size(1) == W, "conv [taps, width]");
  const int64_t taps = cw.size(0);
  TORCH_CHECK(state.is_cuda() && state.scalar_type() == at::kFloat && state.dim() == 2 && state.is_contiguous() &&
                  state.size(1) >= taps * W && state.size(1) % 4 == 0,
              "state f32 [slots, >= taps * width]");
  check_aligned(state, "state");
  RgLruParams p{};
  p.yx = yx.data_ptr();
  p.ld = (int)yx.stride(0);
  p.yb = f32p(yb, W, "yb");
  p.xb = f32p(xb, W, "xb");
  p.cw = f32p(cw, taps * W, "conv");
  p.cb = f32p(cb, W, "conv bias");
  p.taps = (int)taps;
  p.gw = frag(gw, f32, 2 * W * bs, "gates");
  p.rb = f32p(rb, W, "rb");
  p.ib = f32p(ib, W, "ib");
  p.decay = f32p(decay, W, "decay");
  p.nb = (int)nb;
  p.bs = (int)bs;
  p.rows = (int)rows;
  p.f32 = f32;
  p.seq_ids = i32p(seq_ids, rows, "seq_ids");
  p.positions = i32p(positions, rows, "positions");
  p.slots = i64p(slots, rows, "slots");
  p.state = state.data_ptr<float>();
  p.state_ld = state.stride(0);
  p.out = out.data_ptr();
  p.ldo = (int)out.stride(0);
  if (!chunks.has_value()) {
    TORCH_CHECK(rows <= 64, "rows form: at most 64 rows");
    check_rc(vwa_rglru_rows(&p, cur_stream(yx)), "rglru_rows");
    return;
  }
  TORCH_CHECK(chunks->dim() == 2 && chunks->size(1) == 4 && chunks->size(0) >= 1, "chunks int32 [n, 4]");
  p.chunks = i32p(*chunks, chunks->numel(), "chunks");
  p.n_chunks = (int)chunks->size(0);
  TORCH_CHECK(scratch.has_value() && u.has_value(), "scan form needs scratch and u");
  check_t(*u, f32, "u");
  TORCH_CHECK(u->is_contiguous() && u->numel() >= rows * W, "u [rows, width]");
  p.u = u->data_ptr();
  float* s = f32p(*scratch, 3 * (int64_t)p.n_chunks * W, "scratch");
  p.cA = s;
  p.cB = s + (size_t)p.n_chunks * W;
  p.cS = s + (size_t)2 * p.n_chunks * W;
  check_rc(vwa_rglru_scan(&p, cur_stream(yx)), "rglru_scan");
}

HeadLinearParams lin_params(const Tensor& x, int64_t xs, const Tensor& w, int64_t nb, int64_t N, int64_t K, const Tensor& y,
                            int64_t ys, int64_t rows, const OptTensor& row_list = c10::nullopt) {
  const bool f32 = t_is_f32(x, "x");
  TORCH_CHECK(nb >= 1 && N >= 16 && N % 16 == 0 && K >= 32 && K % 32 == 0 && xs >= 0 && ys >= N, "head_linear sizes");
  check_rows(x, rows, (nb - 1) * xs + K, "x");
  check_aligned(x, "x");
  TORCH_CHECK(x.stride(0) % 8 == 0 && xs % 8 == 0, "x rows and heads must be 16-byte aligned");
  check_t(y, f32, "y");
  check_rows(y, rows, (nb - 1) * ys + N, "y");
  HeadLinearParams p{};
  if (row_list.has_value()) {
    p.row_list = i32p(*row_list, 1, "row_list");
    rows = row_list->numel();
  }
  p.x = x.data_ptr();
  p.ldx = (int)x.stride(0);
  p.xs = (int)xs;
  p.w = frag(w, f32, nb * N * K, "w");
  p.nb = (int)nb;
  p.N = (int)N;
  p.K = (int)K;
  p.rows = (int)rows;
  p.f32 = f32;
  p.y = y.data_ptr();
  p.ldy = (int)y.stride(0);
  p.ys = (int)ys;
  return p;
}

// row_list: the rows of x and y it serves (entries below both tensors' rows)
void head_linear(Tensor x, int64_t xs, Tensor w, int64_t nb, int64_t N, int64_t K, Tensor y, int64_t ys, OptTensor row_list) {
  c10::DeviceGuard g(x.device());
  const HeadLinearParams p = lin_params(x, xs, w, nb, N, K, y, ys, y.size(0), row_list);
  check_rc(vwa_head_linear(&p, cur_stream(x)), "head_linear");
}

// x rows [q: H (dim_p + rot_p) | latent rank_p | key part rot_p | ..]; cache [blocks, 1, block_size, rank_p + rot_p] (none: the
// layer reads another layer's)
LatentRowsParams row_params(const Tensor& x, int64_t H, int64_t dim_p, int64_t rot_p, const Tensor& rope, const Tensor& positions,
                            const Tensor& slots, const Tensor& q_out, int64_t q_head, int64_t q_at, const OptTensor& norm, double eps,
                            const OptTensor& cache) {
  const bool f32 = t_is_f32(x, "x");
  const int64_t rows = q_out.size(0);
  TORCH_CHECK(rope.is_cuda() && rope.scalar_type() == at::kFloat && rope.is_contiguous() && rope.dim() == 3 && rope.size(0) >= 1 &&
                  rope.size(1) >= 1 && rope.size(1) * 2 <= rot_p && rope.size(2) == 2,
              "rope table f32 [max_pos, rot / 2, 2]");
  TORCH_CHECK(H >= 1 && q_head >= rot_p && q_at >= 0, "head layout");
  check_t(q_out, f32, "q_out");
  check_rows(q_out, rows, (H - 1) * q_head + q_at + rot_p, "q_out");
  LatentRowsParams p{};
  p.has_kv = cache.has_value();
  int64_t cols = H * (dim_p + rot_p);
  if (p.has_kv) {
    const Tensor& c = *cache;
    check_t(c, f32, "cache");
    TORCH_CHECK(c.dim() == 4 && c.size(1) == 1 && c.stride(3) == 1 && c.stride(2) == c.size(3) && c.size(3) > rot_p,
                "cache [blocks, 1, block_size, rank_p + rot_p]");
    p.rank_p = (int)(c.size(3) - rot_p);
    p.block_size = (int)c.size(2);
    p.cache = c.data_ptr();
    p.c_sb = c.stride(0);
    TORCH_CHECK(norm.has_value() && norm->numel() >= 1 && norm->numel() <= p.rank_p, "norm [rank]");
    p.rank = (int)norm->numel();
    p.norm = f32p(*norm, p.rank, "norm");
    cols += p.rank_p + rot_p;
  } else {
    p.rank = p.rank_p = p.block_size = 1;
  }
  check_rows(x, rows, cols, "x");
  p.x = x.data_ptr();
  p.ldx = (int)x.stride(0);
  p.rows = (int)rows;
  p.H = (int)H;
  p.f32 = f32;
  p.dim_p = (int)dim_p;
  p.rot_p = (int)rot_p;
  p.rot = (int)rope.size(1) * 2;
  p.rope = rope.data_ptr<float>();
  p.max_pos = (int)rope.size(0);
  p.positions = i32p(positions, rows, "positions");
  p.slots = i64p(slots, rows, "slots");
  p.q_out = q_out.data_ptr();
  p.ldq = (int)q_out.stride(0);
  p.q_head = (int)q_head;
  p.q_at = (int)q_at;
  p.eps = (float)eps;
  return p;
}

void latent_rows(Tensor x, int64_t H, int64_t dim_p, int64_t rot_p, Tensor rope, Tensor positions, Tensor slots, Tensor q_out,
                 int64_t q_head, int64_t q_at, OptTensor norm, double eps, OptTensor cache) {
  c10::DeviceGuard g(x.device());
  const LatentRowsParams p = row_params(x, H, dim_p, rot_p, rope, positions, slots, q_out, q_head, q_at, norm, eps, cache);
  check_rc(vwa_latent_rows(&p, cur_stream(x)), "latent_rows");
}

// latent_rows into q_out [rows, H (rank_p + rot_p)] and its first rank_p columns per head = uk_h . q_h
void latent_qkv(Tensor x, int64_t H, int64_t dim_p, int64_t rot_p, int64_t rank_p, Tensor rope, Tensor positions, Tensor slots,
                Tensor q_out, OptTensor norm, double eps, OptTensor cache, Tensor uk) {
  c10::DeviceGuard g(x.device());
  const int64_t dk = rank_p + rot_p;
  const LatentRowsParams p = row_params(x, H, dim_p, rot_p, rope, positions, slots, q_out, dk, rank_p, norm, eps, cache);
  TORCH_CHECK(!p.has_kv || p.rank_p == rank_p, "cache rows hold rank_p + rot_p");
  const HeadLinearParams q = lin_params(x, dim_p + rot_p, uk, H, rank_p, dim_p, q_out, dk, q_out.size(0));
  check_rc(vwa_latent_qkv(&p, &q, cur_stream(x)), "latent_qkv");
}

void latent_attention(Tensor q, Tensor cache, Tensor table, Tensor positions, Tensor seq_ids, Tensor slots, OptTensor row_list,
                      int64_t n_rows, int64_t H, int64_t rank_p, double scale, int64_t nch, Tensor part, Tensor stat) {
  c10::DeviceGuard g(q.device());
  LatentAttnParams p{};
  const bool f32 = t_is_f32(q, "q");
  check_t(cache, f32, "cache");
  TORCH_CHECK(cache.dim() == 4 && cache.size(1) == 1 && cache.stride(3) == 1 && cache.stride(2) == cache.size(3) &&
                  cache.size(3) > rank_p && cache.stride(0) % 8 == 0,
              "cache [blocks, 1, block_size, rank_p + rot_p]");
  check_aligned(cache, "cache");
  const int64_t dk = cache.size(3), total = row_list.has_value() ? q.size(0) : n_rows;
  check_rows(q, total, H * dk, "q");
  check_aligned(q, "q");
  TORCH_CHECK(n_rows >= 1 && H >= 1 && nch >= 1, "sizes");
  TORCH_CHECK(table.is_cuda() && table.scalar_type() == at::kInt && table.dim() == 2 && table.stride(1) == 1, "block table int32");
  p.q = q.data_ptr();
  p.ldq = (int)q.stride(0);
  p.cache = cache.data_ptr();
  p.c_sb = cache.stride(0);
  p.block_table = table.data_ptr<int>();
  p.table_stride = (int)table.stride(0);
  p.block_size = (int)cache.size(2);
  p.positions = i32p(positions, total, "positions");
  p.seq_ids = i32p(seq_ids, total, "seq_ids");
  p.slots = i64p(slots, total, "slots");
  if (row_list.has_value()) p.row_list = i32p(*row_list, n_rows, "row_list");
  p.rows = (int)n_rows;
  p.H = (int)H;
  p.rank_p = (int)rank_p;
  p.rot_p = (int)(dk - rank_p);
  p.f32 = f32;
  p.scale = (float)scale;
  p.nch = (int)nch;
  p.part = f32p(part, n_rows * nch * H * rank_p, "part");
  p.stat = f32p(stat, n_rows * nch * H * 2, "stat");
  check_rc(vwa_latent_attention(&p, cur_stream(q)), "latent_attention");
}

void latent_out(Tensor part, Tensor stat, int64_t nch, Tensor slots, OptTensor row_list, int64_t n_rows, int64_t H, int64_t rank_p,
                Tensor sink, Tensor w, Tensor gate, Tensor out) {
  c10::DeviceGuard g(out.device());
  LatentOutParams p{};
  const bool f32 = t_is_f32(out, "out");
  const int64_t total = row_list.has_value() ? out.size(0) : n_rows;
  TORCH_CHECK(H >= 1 && rank_p >= 32 && n_rows >= 1 && nch >= 1 && w.numel() % (H * rank_p * 16) == 0, "sizes");
  const int64_t vd = w.numel() / (H * rank_p);
  check_rows(out, total, H * vd, "out");
  check_t(gate, f32, "gate");
  check_rows(gate, total, H * vd, "gate");
  p.part = f32p(part, n_rows * nch * H * rank_p, "part");
  p.stat = f32p(stat, n_rows * nch * H * 2, "stat");
  p.nch = (int)nch;
  p.slots = i64p(slots, total, "slots");
  if (row_list.has_value()) p.row_list = i32p(*row_list, n_rows, "row_list");
  p.rows = (int)n_rows;
  p.H = (int)H;
  p.rank_p = (int)rank_p;
  p.vd = (int)vd;
  p.f32 = f32;
  p.sink = f32p(sink, H, "sink");
  p.w = frag(w, f32, H * vd * rank_p, "w");
  p.gate = gate.data_ptr();
  p.ldg = (int)gate.stride(0);
  p.out = out.data_ptr();
  p.ldo = (int)out.stride(0);
  check_rc(vwa_latent_out(&p, cur_stream(out)), "latent_out");
}

// context rows of segs [n, 3] (block-table row, first key, keys of the run) -> lat [64 n, kp], krot [64 n, rot_p]
void latent_gather(Tensor cache, Tensor table, Tensor segs, Tensor lat, Tensor krot) {
  c10::DeviceGuard g(cache.device());
  LatentPrefillParams p{};
  for (const Tensor* t : {&cache, &lat, &krot}) {
    check_bf16(*t, "cache / lat / krot");
    check_aligned(*t, "cache / lat / krot");
  }
  TORCH_CHECK(segs.dim() == 2 && segs.size(1) == 3 && segs.size(0) >= 1, "segs int32 [n, 3]");
  const int64_t n = segs.size(0), rot_p = krot.size(1);
  TORCH_CHECK(lat.dim() == 2 && krot.dim() == 2 && lat.is_contiguous() && krot.is_contiguous() && lat.size(0) >= 64 * n && krot.size(0) >= 64 * n,
              "lat / krot [64 n, ..]");
  TORCH_CHECK(cache.dim() == 4 && cache.size(1) == 1 && cache.stride(3) == 1 && cache.stride(2) == cache.size(3) &&
                  cache.size(3) > rot_p && lat.size(1) >= cache.size(3) - rot_p && cache.stride(0) % 8 == 0,
              "cache [blocks, 1, block_size, rank_p + rot_p]");
  TORCH_CHECK(table.is_cuda() && table.scalar_type() == at::kInt && table.dim() == 2 && table.stride(1) == 1, "block table int32");
  p.cache = cache.data_ptr();
  p.c_sb = cache.stride(0);
  p.block_table = table.data_ptr<int>();
  p.table_stride = (int)table.stride(0);
  p.block_size = (int)cache.size(2);
  p.segs = i32p(segs, 3 * n, "segs");
  p.n_segs = (int)n;
  p.rot_p = (int)rot_p;
  p.rank_p = (int)(cache.size(3) - rot_p);
  p.kp = (int)lat.size(1);
  p.lat = bfp_mut(lat);
  p.krot = bfp_mut(krot);
  check_rc(vwa_latent_gather(&p, cur_stream(cache)), "latent_gather");
}

// tiles [n, 4]: first row, rows, row of its run's key 0 in kv, position of the first row (all inside the tensors)
void latent_prefill(Tensor y, Tensor q, int64_t H, int64_t dim_p, int64_t q_head, int64_t q_at, Tensor kv, Tensor krot, Tensor tiles,
                    double scale, Tensor sink, Tensor gate, int64_t vd, Tensor out) {
  c10::DeviceGuard g(y.device());
  LatentPrefillParams p{};
  for (const Tensor* t : {&y, &q, &kv, &krot, &gate, &out}) {
    check_bf16(*t, "operand");
    TORCH_CHECK(t->dim() == 2 && t->stride(1) == 1, "operands must be 2-D with contiguous columns");
  }
  for (const Tensor* t : {&y, &q, &kv, &krot}) check_aligned(*t, "operand");
  const int64_t rows = out.size(0), rot_p = krot.size(1), cols = kv.size(1) - H * dim_p;
  TORCH_CHECK(H >= 1 && cols > 0 && cols % H == 0 && krot.is_contiguous(), "kv [T, H (dim_p + vdk)]");
  check_rows(y, rows, H * (dim_p + rot_p), "y");
  check_rows(q, rows, (H - 1) * q_head + q_at + rot_p, "q");
  check_rows(gate, rows, H * vd, "gate");
  check_rows(out, rows, H * vd, "out");
  TORCH_CHECK(((reinterpret_cast<uintptr_t>(gate.data_ptr()) | reinterpret_cast<uintptr_t>(out.data_ptr())) & 7) == 0,
              "gate / out rows must be 8-byte aligned");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 4 && tiles.size(0) >= 1, "tiles int32 [n, 4]");
  p.q_tiles = i32p(tiles, tiles.numel(), "tiles");
  p.n_tiles = (int)tiles.size(0);
  p.H = (int)H;
  p.dim_p = (int)dim_p;
  p.rot_p = (int)rot_p;
  p.vdk = (int)(cols / H);
  p.vd = (int)vd;
  p.scale = (float)scale;
  p.qn = y.data_ptr();
  p.ldqn = (int)y.stride(0);
  p.qr = q.data_ptr();
  p.ldqr = (int)q.stride(0);
  p.qr_head = (int)q_head;
  p.qr_at = (int)q_at;
  p.kv = kv.data_ptr();
  p.ldkv = (int)kv.stride(0);
  p.krot = bfp_mut(krot);
  p.sink = f32p(sink, H, "sink");
  p.gate = gate.data_ptr();
  p.ldg = (int)gate.stride(0);
  p.out = out.data_ptr();
  p.ldo = (int)out.stride(0);
  check_rc(vwa_latent_prefill(&p, cur_stream(y)), "latent_prefill");
}

void moe_route(Tensor h, Tensor w, int64_t E, int64_t top, Tensor slots, Tensor wts, Tensor ids, int64_t tile, Tensor tiles,
               Tensor order, Tensor ticket) {
  c10::DeviceGuard g(h.device());
  MoeRouteParams p{};
  const bool f32 = t_is_f32(h, "h");
  const int64_t rows = h.size(0), K = h.size(1);
  TORCH_CHECK(E >= 1 && top >= 1 && top <= E && K % 32 == 0 && tile >= 1 && rows >= 1, "router sizes");
  check_rows(h, rows, K, "h");
  check_aligned(h, "h");
  TORCH_CHECK(h.stride(0) % 8 == 0, "h rows must be 16-byte aligned");
  p.h = h.data_ptr();
  p.ldh = (int)h.stride(0);
  p.K = (int)K;
  p.w = frag(w, f32, (E + 15) / 16 * 16 * K, "router");
  p.rows = (int)rows;
  p.E = (int)E;
  p.top = (int)top;
  p.f32 = f32;
  p.slots = i64p(slots, rows, "slots");
  p.wts = f32p(wts, rows * top, "wts");
  p.ids = const_cast<int*>(i32p(ids, rows * top, "ids"));
  p.tile = (int)tile;
  TORCH_CHECK(tiles.numel() >= 4, "tiles");
  p.max_tiles = (int)((tiles.numel() - 1) / 3);
  p.tiles = const_cast<int*>(i32p(tiles, 4, "tiles"));
  p.order = const_cast<int*>(i32p(order, p.max_tiles * tile, "order"));
  p.ticket = const_cast<int*>(i32p(ticket, 1, "ticket"));
  check_rc(vwa_moe_route(&p, cur_stream(h)), "moe_route");
}

// gate / up (down false): x [rows, K], y [>= places, N / 2]; down: x [>= places, K], y [rows * top, N]
void moe_gemm(Tensor x, Tensor w, int64_t rows, int64_t top, bool down, Tensor wts, int64_t tile, Tensor tiles, Tensor order, Tensor y) {
  c10::DeviceGuard g(x.device());
  MoeGemmParams p{};
  const bool f32 = t_is_f32(x, "x");
  check_t(w, f32, "w");
  check_t(y, f32, "y");
  TORCH_CHECK(w.dim() == 3 && w.is_contiguous(), "w [experts, N, K] (tiled)");
  const int64_t N = w.size(1), K = w.size(2);
  p.max_tiles = (int)((tiles.numel() - 1) / 3);
  const int64_t places = p.max_tiles * tile;
  check_rows(x, down ? places : rows, K, "x");
  check_rows(y, down ? rows * top : places, down ? N : N / 2, "y");
  check_aligned(x, "x");
  check_aligned(w, "w");
  TORCH_CHECK(x.stride(0) % 8 == 0, "x rows must be 16-byte aligned");
  p.x = x.data_ptr();
  p.ldx = (int)x.stride(0);
  p.w = w.data_ptr();
  p.w_expert = N * K;
  p.N = (int)N;
  p.K = (int)K;
  p.top = (int)top;
  p.f32 = f32;
  p.down = down;
  p.wts = f32p(wts, rows * top, "wts");
  p.tiles = i32p(tiles, 4, "tiles");
  p.order = i32p(order, places, "order");
  p.tile = (int)tile;
  p.x_rows = (int)(down ? places : rows);
  if (tile > 32) {
    check_aligned(y, "y");
    TORCH_CHECK(y.stride(0) % 8 == 0, "y rows must be 16-byte aligned");
  }
  p.y = y.data_ptr();
  p.ldy = (int)y.stride(0);
  check_rc(vwa_moe_gemm(&p, cur_stream(x)), "moe_gemm");
}

}  // namespace

void bind_mixers(py::module_& m) {
  m.def("rglru", &rglru, py::arg("yx"), py::arg("yb"), py::arg("xb"), py::arg("cw"), py::arg("cb"), py::arg("gw"), py::arg("rb"),
        py::arg("ib"), py::arg("decay"), py::arg("nb"), py::arg("seq_ids"), py::arg("positions"), py::arg("slots"), py::arg("state"),
        py::arg("out"), py::arg("chunks") = py::none(), py::arg("scratch") = py::none(), py::arg("u") = py::none());
  m.def("head_linear", &head_linear, py::arg("x"), py::arg("xs"), py::arg("w"), py::arg("nb"), py::arg("N"), py::arg("K"), py::arg("y"),
        py::arg("ys"), py::arg("row_list") = py::none());
  m.def("latent_rows", &latent_rows);
  m.def("latent_qkv", &latent_qkv);
  m.def("latent_attention", &latent_attention);
  m.def("latent_out", &latent_out);
  m.def("latent_prefill_fits", [](int64_t dim_p, int64_t rot_p, int64_t vdk) { return vwa_latent_prefill_fits((int)dim_p, (int)rot_p, (int)vdk) != 0; });
  m.def("latent_gather", &latent_gather);
  m.def("latent_prefill", &latent_prefill);
  m.def("moe_route", &moe_route);
  m.def("moe_gemm", &moe_gemm);
}
