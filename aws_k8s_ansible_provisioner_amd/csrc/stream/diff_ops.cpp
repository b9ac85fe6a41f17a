// torch custom-op registrations (namespace `akap_stream`, a fragment beside stream_ops.cpp) of the
// kernels in diff.hip and diff_mfma.hip.
//
// Like the other ops: every op launches on the caller's current HIP stream, allocates nothing and
// never synchronises (hipGraph-capturable).  Operand shapes are checked here, on the host, against
// what the kernels index.
#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>
#include <c10/core/DeviceGuard.h>

#include "stream.h"

namespace {

using at::Tensor;

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

#define CHECK_GPU(x) TORCH_CHECK((x).is_cuda(), #x " must be a GPU tensor")
#define CHECK_LAST_CONTIG(x) TORCH_CHECK((x).stride(-1) == 1, #x " must have unit last stride")
#define CHECK_CONTIG(x) TORCH_CHECK((x).is_contiguous(), #x " must be contiguous")
#define CHECK_F32(x) TORCH_CHECK((x).scalar_type() == at::kFloat, #x " must be fp32")
#define CHECK_I32(x) TORCH_CHECK((x).scalar_type() == at::kInt, #x " must be int32")

bool is_f32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16, name,
              " must be bf16 or fp32");
  return t.scalar_type() == at::kFloat;
}

const float* f32_vec(const std::optional<Tensor>& t, int64_t n, const char* name) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->scalar_type() == at::kFloat && t->is_contiguous() &&
                  t->numel() == n, name, " must be a contiguous fp32 GPU tensor of ", n, " entries");
  return t->data_ptr<float>();
}

void layer_norm_step(Tensor out, Tensor x, Tensor ya, std::optional<Tensor> yb,
                     std::optional<Tensor> post_w, std::optional<Tensor> next_w, double eps,
                     bool fresh) {
  CHECK_GPU(out); CHECK_GPU(x); CHECK_GPU(ya); CHECK_F32(x); CHECK_CONTIG(x);
  CHECK_LAST_CONTIG(out); CHECK_LAST_CONTIG(ya);
  TORCH_CHECK(x.dim() == 2 && out.dim() == 2 && out.sizes() == x.sizes() && ya.dim() == 2 &&
                  ya.sizes() == x.sizes(), "layer_norm_step: shapes");
  akap_stream::LayerNormStepParams p{};
  p.rows = x.size(0);
  p.d = x.size(1);
  TORCH_CHECK(p.d >= 1 && p.d <= 12000, "layer_norm_step: rows of at most 12000 entries");
  TORCH_CHECK(out.data_ptr() != x.data_ptr(), "layer_norm_step: out must not alias x");
  p.out = out.data_ptr(); p.out_stride = out.stride(0);
  p.x = x.data_ptr<float>();
  p.ya = ya.data_ptr(); p.ya_stride = ya.stride(0); p.ya_f32 = is_f32(ya, "ya");
  if (yb.has_value()) {
    CHECK_GPU(*yb); CHECK_LAST_CONTIG(*yb);
    TORCH_CHECK(yb->dim() == 2 && yb->sizes() == x.sizes(), "layer_norm_step: yb shape");
    p.yb = yb->data_ptr(); p.yb_stride = yb->stride(0); p.yb_f32 = is_f32(*yb, "yb");
  }
  p.post_w = f32_vec(post_w, p.d, "post_w");
  p.next_w = f32_vec(next_w, p.d, "next_w");
  p.eps = (float)eps;
  p.fresh = fresh;
  const c10::DeviceGuard g(x.device());
  akap_stream::launch_layer_norm_step(p, is_f32(out, "out"), cur_stream());
}

void clamped_glu(Tensor out, Tensor gu, std::optional<Tensor> ids, std::optional<Tensor> w,
                 int64_t experts, double limit, int64_t shared_ff, double shared_limit,
                 std::optional<Tensor> shared_w, double alpha) {
  CHECK_GPU(out); CHECK_GPU(gu); CHECK_LAST_CONTIG(out); CHECK_LAST_CONTIG(gu);
  TORCH_CHECK(out.dim() == 2 && gu.dim() == 2 && out.size(0) == gu.size(0) &&
                  gu.size(1) == 2 * out.size(1) && out.scalar_type() == gu.scalar_type(),
              "clamped_glu: gu must be [T, 2 n] for out [T, n], of one type");
  TORCH_CHECK(experts >= 0 && shared_ff >= 0 && shared_ff <= out.size(1) && limit >= 0 &&
                  shared_limit >= 0, "clamped_glu: experts / shared_ff / limits");
  const int64_t n = out.size(1) - shared_ff;
  TORCH_CHECK(experts > 0 ? n % experts == 0 : n == 0, "clamped_glu: columns per expert");
  akap_stream::ClampedGluParams p{};
  p.out = out.data_ptr(); p.out_stride = out.stride(0);
  p.gu = gu.data_ptr(); p.gu_stride = gu.stride(0);
  p.rows = out.size(0);
  p.E = experts; p.F = experts > 0 ? n / experts : 0; p.Fs = shared_ff;
  if (p.F == 0) p.E = 0;
  p.limit = (float)limit; p.shared_limit = (float)shared_limit; p.alpha = (float)alpha;
  if (ids.has_value()) {
    TORCH_CHECK(w.has_value(), "clamped_glu: ids need w");
    CHECK_GPU(*ids); CHECK_I32(*ids); CHECK_CONTIG(*ids); CHECK_GPU(*w); CHECK_F32(*w);
    CHECK_CONTIG(*w);
    TORCH_CHECK(ids->dim() == 2 && ids->size(0) == p.rows && w->sizes() == ids->sizes(),
                "clamped_glu: ids / w [T, top]");
    p.ids = ids->data_ptr<int32_t>(); p.w = w->data_ptr<float>(); p.top = ids->size(1);
  }
  p.shared_w = f32_vec(shared_w, p.rows, "shared_w");
  TORCH_CHECK((out.size(1) + 255) / 256 <= 65535, "clamped_glu: too many columns");
  const c10::DeviceGuard g(out.device());
  akap_stream::launch_clamped_glu(p, is_f32(out, "out"), cur_stream());
}

akap_stream::DiffAttnParams diff_params(const Tensor& out, const Tensor& q, const Tensor& k_cache,
                                        const Tensor& v_cache, const Tensor& block_tables,
                                        const Tensor& seq_lens, const std::optional<Tensor>& gate,
                                        int64_t H, double lam, double diff, double scale,
                                        int64_t chunk, double eps) {
  CHECK_GPU(out); CHECK_GPU(q); CHECK_GPU(k_cache); CHECK_GPU(v_cache); CHECK_GPU(block_tables);
  CHECK_GPU(seq_lens);
  CHECK_LAST_CONTIG(out); CHECK_LAST_CONTIG(q); CHECK_CONTIG(k_cache); CHECK_CONTIG(v_cache);
  CHECK_LAST_CONTIG(block_tables); CHECK_CONTIG(seq_lens); CHECK_I32(block_tables);
  CHECK_I32(seq_lens);
  TORCH_CHECK(k_cache.scalar_type() == q.scalar_type() && v_cache.scalar_type() == q.scalar_type() &&
                  out.scalar_type() == q.scalar_type(), "diff_attention: dtypes differ");
  is_f32(q, "q");
  TORCH_CHECK(k_cache.dim() == 4 && v_cache.dim() == 5 && k_cache.size(3) % 2 == 0 &&
                  v_cache.size(0) == k_cache.size(0) && v_cache.size(1) == k_cache.size(1) &&
                  v_cache.size(2) * 8 == k_cache.size(2) && v_cache.size(4) == 8,
              "diff_attention: K [NB, G, BS, 2 D], V [NB, G, BS / 8, Dv, 8]");
  akap_stream::DiffAttnParams p{};
  p.NB = k_cache.size(0); p.G = k_cache.size(1); p.BS = k_cache.size(2);
  p.D = k_cache.size(3) / 2; p.Dv = v_cache.size(3);
  p.H = H;
  p.T = q.size(0);
  TORCH_CHECK(H > 0 && p.G > 0 && H % p.G == 0 && p.D > 0 && p.Dv > 0 && H <= 65535,
              "diff_attention: heads");
  TORCH_CHECK((int64_t)p.NB * p.G * p.BS < (1LL << 31), "diff_attention: cache rows");
  TORCH_CHECK(q.dim() == 2 && q.size(1) == H * 2 * p.D && out.dim() == 2 && out.size(0) == p.T &&
                  out.size(1) == H * p.Dv, "diff_attention: q [T, H 2 D], out [T, H Dv]");
  TORCH_CHECK(block_tables.dim() == 2 && block_tables.size(0) >= seq_lens.numel() &&
                  block_tables.stride(0) == block_tables.size(1), "diff_attention: block tables");
  p.out = out.data_ptr(); p.out_stride = out.stride(0);
  p.q = q.data_ptr(); p.q_stride = q.stride(0);
  p.k_cache = k_cache.data_ptr(); p.v_cache = v_cache.data_ptr();
  p.block_tables = block_tables.data_ptr<int32_t>(); p.max_blocks = block_tables.size(1);
  p.seq_lens = seq_lens.data_ptr<int32_t>(); p.B = seq_lens.numel();
  if (gate.has_value()) {
    CHECK_GPU(*gate); CHECK_LAST_CONTIG(*gate);
    TORCH_CHECK(gate->sizes() == out.sizes() && gate->scalar_type() == q.scalar_type(),
                "diff_attention: gate");
    p.gate = gate->data_ptr(); p.gate_stride = gate->stride(0);
  }
  p.lam = (float)lam; p.out_mult = (float)(1.0 - diff); p.scale = (float)scale;
  p.eps = (float)eps; p.chunk = (int)chunk;
  TORCH_CHECK(chunk >= 0, "diff_attention: chunk");
  p.num_parts = 1;
  return p;
}

const int32_t* starts(const Tensor& q_start, int B) {
  CHECK_GPU(q_start); CHECK_CONTIG(q_start); CHECK_I32(q_start);
  TORCH_CHECK(q_start.numel() >= B + 1, "diff_attention: q_start");
  return q_start.data_ptr<int32_t>();
}

void diff_attention(Tensor out, Tensor q, Tensor k_cache, Tensor v_cache, Tensor block_tables,
                    Tensor seq_lens, std::optional<Tensor> q_start, Tensor positions,
                    std::optional<Tensor> gate, int64_t heads, double lam, double diff,
                    double scale, int64_t chunk, double eps) {
  auto p = diff_params(out, q, k_cache, v_cache, block_tables, seq_lens, gate, heads, lam, diff,
                       scale, chunk, eps);
  CHECK_GPU(positions); CHECK_CONTIG(positions);
  TORCH_CHECK(positions.scalar_type() == at::kLong && positions.numel() >= p.T,
              "diff_attention: int64 positions");
  TORCH_CHECK(p.Dv <= 512 && p.D <= 1024, "diff_attention: heads of at most 1024 / 512 entries");
  p.positions = positions.data_ptr<int64_t>();
  if (q_start.has_value()) p.q_start = starts(*q_start, p.B);
  else TORCH_CHECK(p.T <= p.B, "diff_attention: a row per sequence");
  const c10::DeviceGuard g(q.device());
  akap_stream::launch_diff_attention(p, is_f32(q, "q"), cur_stream());
}

void check_mfma(const akap_stream::DiffAttnParams& p, const Tensor& q) {
  TORCH_CHECK(q.scalar_type() == at::kBFloat16 &&
                  akap_stream::diff_mfma_supported(p.D, p.Dv, p.BS) && p.scale > 0,
              "diff_attention: sizes of the matrix-core form");
  TORCH_CHECK(p.q_stride % 8 == 0 && (uintptr_t)p.q % 16 == 0 && p.out_stride % 4 == 0 &&
                  (uintptr_t)p.out % 8 == 0 && p.gate_stride % 4 == 0 &&
                  (uintptr_t)p.gate % 8 == 0, "diff_attention: alignment of the matrix-core form");
}

void diff_attention_prefill_mfma(Tensor out, Tensor q, Tensor k_cache, Tensor v_cache,
                                 Tensor block_tables, Tensor seq_lens, Tensor q_start,
                                 Tensor tile_seq, Tensor tile_row, int64_t tile_rows,
                                 std::optional<Tensor> gate, int64_t heads, double lam,
                                 double diff, double scale, int64_t chunk, double eps) {
  auto p = diff_params(out, q, k_cache, v_cache, block_tables, seq_lens, gate, heads, lam, diff,
                       scale, chunk, eps);
  check_mfma(p, q);
  CHECK_GPU(tile_seq); CHECK_GPU(tile_row); CHECK_I32(tile_seq); CHECK_I32(tile_row);
  CHECK_CONTIG(tile_seq); CHECK_CONTIG(tile_row);
  TORCH_CHECK(tile_seq.numel() == tile_row.numel() && tile_rows == 128,
              "diff_attention: a map of 128-token tiles");
  p.q_start = starts(q_start, p.B);
  p.tile_seq = tile_seq.data_ptr<int32_t>(); p.tile_row = tile_row.data_ptr<int32_t>();
  p.num_tiles = tile_seq.numel(); p.tile_rows = tile_rows;
  const c10::DeviceGuard g(q.device());
  akap_stream::launch_diff_prefill_mfma(p, cur_stream());
}

void diff_attention_decode_mfma(Tensor out, Tensor q, Tensor k_cache, Tensor v_cache,
                                Tensor block_tables, Tensor seq_lens, std::optional<Tensor> gate,
                                int64_t heads, double lam, double diff, double scale,
                                int64_t chunk, double eps, std::optional<Tensor> ws_ml,
                                std::optional<Tensor> ws_o, int64_t num_parts) {
  auto p = diff_params(out, q, k_cache, v_cache, block_tables, seq_lens, gate, heads, lam, diff,
                       scale, chunk, eps);
  check_mfma(p, q);
  TORCH_CHECK(p.T == p.B, "diff_attention: one query row per sequence");
  TORCH_CHECK(num_parts >= 1 && num_parts <= 64, "diff_attention: at most 64 partitions");
  p.num_parts = num_parts;
  if (num_parts > 1) {
    TORCH_CHECK(ws_ml.has_value() && ws_o.has_value(), "diff_attention: workspace");
    CHECK_GPU(*ws_ml); CHECK_GPU(*ws_o); CHECK_F32(*ws_ml); CHECK_F32(*ws_o);
    CHECK_CONTIG(*ws_ml); CHECK_CONTIG(*ws_o);
    const int64_t n = (int64_t)p.B * p.H * 2 * num_parts;
    TORCH_CHECK(ws_ml->numel() >= 2 * n && ws_o->numel() >= n * p.Dv &&
                    (uintptr_t)ws_o->data_ptr() % 16 == 0, "diff_attention: workspace too small");
    p.ws_ml = ws_ml->data_ptr<float>();
    p.ws_o = ws_o->data_ptr<float>();
  }
  const c10::DeviceGuard g(q.device());
  akap_stream::launch_diff_decode_mfma(p, cur_stream());
}

bool diff_mfma_supported(int64_t D, int64_t Dv, int64_t BS) {
  return akap_stream::diff_mfma_supported((int)D, (int)Dv, (int)BS);
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(akap_stream, m) {
  m.def("layer_norm_step(Tensor(a!) out, Tensor(b!) x, Tensor ya, Tensor? yb, Tensor? post_w, "
        "Tensor? next_w, float eps, bool fresh) -> ()");
  m.def("clamped_glu(Tensor(a!) out, Tensor gu, Tensor? ids, Tensor? w, int experts, float limit, "
        "int shared_ff, float shared_limit, Tensor? shared_w, float alpha) -> ()");
  m.def("diff_attention(Tensor(a!) out, Tensor q, Tensor k_cache, Tensor v_cache, "
        "Tensor block_tables, Tensor seq_lens, Tensor? q_start, Tensor positions, Tensor? gate, "
        "int heads, float lam, float diff, float scale, int chunk, float eps) -> ()");
  m.def("diff_attention_prefill_mfma(Tensor(a!) out, Tensor q, Tensor k_cache, Tensor v_cache, "
        "Tensor block_tables, Tensor seq_lens, Tensor q_start, Tensor tile_seq, Tensor tile_row, "
        "int tile_rows, Tensor? gate, int heads, float lam, float diff, float scale, int chunk, "
        "float eps) -> ()");
  m.def("diff_attention_decode_mfma(Tensor(a!) out, Tensor q, Tensor k_cache, Tensor v_cache, "
        "Tensor block_tables, Tensor seq_lens, Tensor? gate, int heads, float lam, float diff, "
        "float scale, int chunk, float eps, Tensor(b!)? ws_ml, Tensor(c!)? ws_o, int num_parts) "
        "-> ()");
  m.def("diff_mfma_supported(int D, int Dv, int BS) -> bool", &diff_mfma_supported);
}

TORCH_LIBRARY_IMPL(akap_stream, CUDA, m) {
  m.impl("layer_norm_step", &layer_norm_step);
  m.impl("clamped_glu", &clamped_glu);
  m.impl("diff_attention", &diff_attention);
  m.impl("diff_attention_prefill_mfma", &diff_attention_prefill_mfma);
  m.impl("diff_attention_decode_mfma", &diff_attention_decode_mfma);
}
