// torch custom-op registrations (namespace `akap_stream`, a fragment beside stream_ops.cpp) of
// the kernels in recurrence.hip and recurrence_mfma.hip.
//
// Like the other ops: every op launches on the caller's current HIP stream, allocates nothing
// and never synchronises (hipGraph-capturable).  Operand shapes are checked here, on the host,
// against what the kernels index.
#include <torch/library.h>
#include <ATen/ATen.h>
#include <c10/hip/HIPStream.h>
#include <c10/core/DeviceGuard.h>

#include "stream.h"

namespace {

using at::Tensor;

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

#define CHECK_GPU(x) TORCH_CHECK((x).is_cuda(), #x " must be a GPU tensor")
#define CHECK_CONTIG(x) TORCH_CHECK((x).is_contiguous(), #x " must be contiguous")

bool is_f32(const Tensor& t, const char* name) {
  TORCH_CHECK(t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16, name,
              " must be bf16 or fp32");
  return t.scalar_type() == at::kFloat;
}

float* f32_ptr(const Tensor& t, int64_t n, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == at::kFloat && t.is_contiguous() && t.numel() == n,
              name, " must be a contiguous fp32 GPU tensor of ", n, " entries");
  return t.data_ptr<float>();
}

void rows_of(const Tensor& t, int64_t T, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.size(0) == T && t.stride(1) == 1, name,
              " must be a GPU matrix of one row per token with unit last stride");
}

void norm_gate(Tensor out, Tensor y, Tensor gate, Tensor w, int64_t groups, double eps, int64_t act,
               std::optional<Tensor> den, std::optional<Tensor> floor) {
  CHECK_GPU(y);
  TORCH_CHECK(y.dim() == 2 && y.scalar_type() == at::kFloat && y.is_contiguous(),
              "norm_gate: y must be contiguous fp32 [T, n]");
  const int64_t T = y.size(0), n = y.size(1);
  rows_of(out, T, "out");
  rows_of(gate, T, "gate");
  TORCH_CHECK(out.size(1) == n && gate.size(1) == n && out.scalar_type() == gate.scalar_type(),
              "norm_gate: shapes / dtypes");
  TORCH_CHECK(groups >= 1 && n % groups == 0, "norm_gate: groups");
  TORCH_CHECK(den.has_value() == floor.has_value(), "norm_gate: den and floor come together");
  const c10::DeviceGuard g(y.device());
  akap_stream::launch_norm_gate(
      out.data_ptr(), (int)out.stride(0), y.data_ptr<float>(), gate.data_ptr(),
      (int)gate.stride(0), f32_ptr(w, n, "w"), den ? f32_ptr(*den, T * groups, "den") : nullptr,
      floor ? f32_ptr(*floor, T * groups, "floor") : nullptr, is_f32(out, "out"), (int)act, (int)T,
      (int)n, (int)groups, (float)eps, cur_stream());
}

// the operands the scan and the chunked form share
akap_stream::RecurrenceParams recurrence_params(
    int64_t mode, const Tensor& qkv, int64_t q_off, int64_t k_off, int64_t v_off, int64_t act,
    const Tensor& proj, int64_t a_off, int64_t b_off, const Tensor& pa,
    const std::optional<Tensor>& pb, double cap, double q_scale, const Tensor& state,
    const std::optional<Tensor>& n_state, const std::optional<Tensor>& m_state,
    const Tensor& seq_slot, const Tensor& positions, const std::optional<Tensor>& q_start,
    int64_t H, int64_t G, int64_t D, int64_t V) {
  CHECK_GPU(qkv); CHECK_GPU(proj); CHECK_GPU(state); CHECK_GPU(seq_slot); CHECK_GPU(positions);
  const int64_t T = qkv.size(0);
  rows_of(qkv, T, "qkv");
  rows_of(proj, T, "proj");
  TORCH_CHECK(mode >= 0 && mode <= 2, "recurrence: mode");
  TORCH_CHECK(qkv.scalar_type() == proj.scalar_type(), "recurrence: dtypes differ");
  TORCH_CHECK(H >= 1 && G >= 1 && H % G == 0 && H <= 65535 &&
                  akap_stream::recurrence_supported((int)D, (int)V),
              "recurrence: heads / sizes (dim at most 1024)");
  const int64_t N = qkv.size(1), P = proj.size(1);
  TORCH_CHECK(q_off >= 0 && k_off >= 0 && v_off >= 0 && q_off + G * D <= N && k_off + G * D <= N &&
                  v_off + H * V <= N, "recurrence: q / k / v outside their rows");
  TORCH_CHECK(mode == akap_stream::kDecay ||
                  (a_off >= 0 && b_off >= 0 && a_off + H <= P && b_off + H <= P),
              "recurrence: gates outside the projection");
  TORCH_CHECK(state.dim() == 4 && state.is_contiguous() && state.scalar_type() == at::kFloat &&
                  state.size(1) == H && state.size(2) == V && state.size(3) == D,
              "recurrence: state must be fp32 [slots, H, V, D]");
  const int64_t slots = state.size(0);
  TORCH_CHECK(seq_slot.scalar_type() == at::kInt && seq_slot.is_contiguous() &&
                  positions.scalar_type() == at::kLong && positions.is_contiguous() &&
                  seq_slot.numel() >= T && positions.numel() >= T,
              "recurrence: seq_slot int32 and positions int64, one per row");
  akap_stream::RecurrenceParams p{};
  p.qkv = qkv.data_ptr(); p.qkv_stride = (int)qkv.stride(0);
  p.q_off = (int)q_off; p.k_off = (int)k_off; p.v_off = (int)v_off; p.act = (int)act;
  p.proj = proj.data_ptr(); p.proj_stride = (int)proj.stride(0);
  p.a_off = (int)a_off; p.b_off = (int)b_off;
  p.pa = f32_ptr(pa, H, "pa");
  TORCH_CHECK(mode == akap_stream::kDecay || pb.has_value(), "recurrence: pb");
  p.pb = pb ? f32_ptr(*pb, H, "pb") : nullptr;
  p.cap = (float)cap; p.q_scale = (float)q_scale;
  p.state = state.data_ptr<float>();
  p.num_slots = (int)slots;
  if (mode == akap_stream::kMatrixMemory) {
    TORCH_CHECK(n_state.has_value() && m_state.has_value() && cap > 0,
                "recurrence: the matrix memory needs n_state, m_state and a cap");
    p.n_state = f32_ptr(*n_state, slots * H * D, "n_state");
    p.m_state = f32_ptr(*m_state, slots * H, "m_state");
  }
  p.seq_slot = seq_slot.data_ptr<int32_t>();
  p.positions = positions.data_ptr<int64_t>();
  p.q_start = nullptr;
  p.num_seqs = (int)T;
  if (q_start.has_value()) {
    TORCH_CHECK(q_start->is_cuda() && q_start->scalar_type() == at::kInt &&
                    q_start->is_contiguous() && q_start->numel() >= 1, "recurrence: q_start");
    p.q_start = q_start->data_ptr<int32_t>();
    p.num_seqs = (int)q_start->numel() - 1;
  }
  p.H = (int)H; p.G = (int)G; p.D = (int)D; p.V = (int)V;
  return p;
}

void recurrence(int64_t mode, Tensor out, std::optional<Tensor> raw, Tensor qkv, int64_t q_off,
                int64_t k_off, int64_t v_off, int64_t act, Tensor proj, int64_t a_off,
                int64_t b_off, Tensor pa, std::optional<Tensor> pb, double cap, double q_scale,
                Tensor state, std::optional<Tensor> n_state, std::optional<Tensor> m_state,
                Tensor norm_w, int64_t g_off, int64_t gate_act, double eps, Tensor seq_slot,
                Tensor positions, std::optional<Tensor> q_start, int64_t H, int64_t G, int64_t D,
                int64_t V, bool step) {
  auto p = recurrence_params(mode, qkv, q_off, k_off, v_off, act, proj, a_off, b_off, pa, pb, cap,
                             q_scale, state, n_state, m_state, seq_slot, positions, q_start, H, G,
                             D, V);
  const int64_t T = qkv.size(0);
  rows_of(out, T, "out");
  TORCH_CHECK(out.size(1) == H * V && out.scalar_type() == qkv.scalar_type(),
              "recurrence: out [T, H V] of qkv's type");
  TORCH_CHECK(g_off >= 0 && g_off + H * V <= proj.size(1), "recurrence: gate outside the projection");
  TORCH_CHECK(raw.has_value() || step || akap_stream::recurrence_fused((int)D, (int)V),
              "recurrence: this head size needs raw");
  p.out = out.data_ptr(); p.out_stride = (int)out.stride(0);
  p.raw = raw ? f32_ptr(*raw, T * H * V, "raw") : nullptr;
  p.g_off = (int)g_off; p.gate_act = (int)gate_act;
  p.norm_w = f32_ptr(norm_w, H * V, "norm_w");
  p.eps = (float)eps;
  const c10::DeviceGuard g(qkv.device());
  if (step) {
    TORCH_CHECK(!q_start.has_value() && akap_stream::recurrence_step_supported((int)D, (int)V) &&
                    ((q_off | k_off | v_off | qkv.stride(0)) & 3) == 0 &&
                    ((uintptr_t)qkv.data_ptr() & 15) == 0,
                "recurrence: the single-row form needs sizes, offsets and strides in fours");
    akap_stream::launch_recurrence_step(p, (int)mode, is_f32(qkv, "qkv"), cur_stream());
    return;
  }
  akap_stream::launch_recurrence(p, (int)mode, is_f32(qkv, "qkv"), cur_stream());
}

// the chunked form over the sequences from first_seq on (their first row is row0, on the host)
void chunk_recurrence(int64_t mode, Tensor raw, Tensor qkv, int64_t q_off, int64_t k_off,
                      int64_t v_off, int64_t act, Tensor proj, int64_t a_off, int64_t b_off,
                      Tensor pa, std::optional<Tensor> pb, double cap, double q_scale,
                      Tensor state, std::optional<Tensor> n_state, std::optional<Tensor> m_state,
                      Tensor seq_slot, Tensor positions, Tensor q_start, int64_t first_seq,
                      int64_t row0, int64_t H, int64_t G, int64_t D, int64_t V,
                      std::optional<Tensor> memory, Tensor halves, Tensor floats) {
  auto p = recurrence_params(mode, qkv, q_off, k_off, v_off, act, proj, a_off, b_off, pa, pb, cap,
                             q_scale, state, n_state, m_state, seq_slot, positions, q_start, H, G,
                             D, V);
  const int64_t T = qkv.size(0);
  TORCH_CHECK(qkv.scalar_type() == at::kBFloat16 && akap_stream::chunk_supported((int)D),
              "chunk_recurrence: bf16 heads of 32 / 64 / 96 / 128 / 256");
  TORCH_CHECK(((q_off | k_off | qkv.stride(0)) & 7) == 0 &&
                  ((uintptr_t)qkv.data_ptr() & 15) == 0, "chunk_recurrence: 16-byte aligned rows");
  TORCH_CHECK(first_seq >= 0 && first_seq < q_start.numel() && row0 >= 0 && row0 <= T,
              "chunk_recurrence: first_seq / row0");
  p.q_start += first_seq;
  p.num_seqs -= (int)first_seq;
  TORCH_CHECK(p.num_seqs <= 65535, "chunk_recurrence: at most 65535 sequences");
  akap_stream::ChunkParams c{};
  p.raw = f32_ptr(raw, T * H * V, "raw");
  c.r = p;
  c.row0 = (int)row0;
  c.num_chunks = (int)((T - row0) / 64 + p.num_seqs);
  if (mode == akap_stream::kMatrixMemory) {
    TORCH_CHECK(memory.has_value(), "chunk_recurrence: the matrix memory needs [4, T, H] floats");
    float* m = f32_ptr(*memory, 4 * T * H, "memory");
    c.la = m; c.lb = m + T * H; c.den = m + 2 * T * H; c.floor = m + 3 * T * H;
  }
  int64_t nh = 0, nf = 0;
  akap_stream::chunk_workspace((int)mode, c.num_chunks, (int)H, (int)G, (int)D, &nh, &nf);
  TORCH_CHECK(halves.is_cuda() && halves.is_contiguous() &&
                  halves.scalar_type() == at::kBFloat16 && halves.numel() >= nh &&
                  ((uintptr_t)halves.data_ptr() & 15) == 0 && floats.is_cuda() &&
                  floats.is_contiguous() && floats.scalar_type() == at::kFloat &&
                  floats.numel() >= nf && ((uintptr_t)floats.data_ptr() & 15) == 0,
              "chunk_recurrence: workspace");
  const c10::DeviceGuard g(qkv.device());
  akap_stream::launch_chunk_recurrence(c, (int)mode, (uint16_t*)halves.data_ptr(),
                                       floats.data_ptr<float>(), cur_stream());
}

bool chunk_supported(int64_t D) { return akap_stream::chunk_supported((int)D); }

std::vector<int64_t> chunk_workspace(int64_t mode, int64_t chunks, int64_t H, int64_t G, int64_t D) {
  int64_t nh = 0, nf = 0;
  akap_stream::chunk_workspace((int)mode, (int)chunks, (int)H, (int)G, (int)D, &nh, &nf);
  return {nh, nf};
}

bool recurrence_step_supported(int64_t D, int64_t V) {
  return akap_stream::recurrence_step_supported((int)D, (int)V);
}

bool recurrence_fused(int64_t D, int64_t V) {
  return akap_stream::recurrence_fused((int)D, (int)V);
}

}  // namespace

TORCH_LIBRARY_FRAGMENT(akap_stream, m) {
  m.def("norm_gate(Tensor(a!) out, Tensor y, Tensor gate, Tensor w, int groups, float eps, int act, "
        "Tensor? den, Tensor? floor) -> ()");
  m.def("recurrence(int mode, Tensor(a!) out, Tensor(b!)? raw, Tensor qkv, int q_off, int k_off, "
        "int v_off, int act, Tensor proj, int a_off, int b_off, Tensor pa, Tensor? pb, float cap, "
        "float q_scale, Tensor(c!) state, Tensor(d!)? n_state, Tensor(e!)? m_state, Tensor norm_w, "
        "int g_off, int gate_act, float eps, Tensor seq_slot, Tensor positions, Tensor? q_start, "
        "int H, int G, int D, int V, bool step) -> ()");
  m.def("chunk_recurrence(int mode, Tensor(a!) raw, Tensor qkv, int q_off, int k_off, int v_off, "
        "int act, Tensor proj, int a_off, int b_off, Tensor pa, Tensor? pb, float cap, "
        "float q_scale, Tensor(b!) state, Tensor(c!)? n_state, Tensor(d!)? m_state, "
        "Tensor seq_slot, Tensor positions, Tensor q_start, int first_seq, int row0, int H, int G, "
        "int D, int V, Tensor(e!)? memory, Tensor(f!) halves, Tensor(g!) floats) -> ()");
  m.def("chunk_supported(int D) -> bool", &chunk_supported);
  m.def("chunk_workspace(int mode, int chunks, int H, int G, int D) -> int[]", &chunk_workspace);
  m.def("recurrence_step_supported(int D, int V) -> bool", &recurrence_step_supported);
  m.def("recurrence_fused(int D, int V) -> bool", &recurrence_fused);
}

TORCH_LIBRARY_IMPL(akap_stream, CUDA, m) {
  m.impl("norm_gate", &norm_gate);
  m.impl("recurrence", &recurrence);
  m.impl("chunk_recurrence", &chunk_recurrence);
}
