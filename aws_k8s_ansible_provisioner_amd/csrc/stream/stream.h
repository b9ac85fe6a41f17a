// Launchers of the fp32-residual-stream kernels (library _C_stream.so, torch.ops.akap_stream).
//
// Activations, weights and the KV cache are bf16 or fp32 (`f32` flags below); norms, rotary
// angles, attention scores / softmax / gates and the residual sum are fp32 in both.  Every size
// (width, heads, GQA ratio, head size, block size) is a run-time argument.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace akap_stream {

void launch_embed_scaled(float* out, const int64_t* ids, const void* table, bool f32, int rows,
                         int d, int vocab, float scale, hipStream_t s);
// x (fp32, contiguous rows of d) += mult * y (y may be null); out = rmsnorm(x) * w
// (bias: d values of y's type added to every row of y, or null)
void launch_add_norm(void* out, bool out_f32, float* x, const void* y, bool y_f32, int y_stride,
                     const void* bias, float mult, const float* w, int rows, int d,
                     int out_stride, float eps, hipStream_t s);
// act 0: relu(x)^2, 1: gelu in its tanh form
void launch_activation(void* out, const void* x, bool f32, int act, int rows, int F, int x_stride,
                       int out_stride, hipStream_t s);

struct ProjParams {
  const void* proj;   // [T, N] fused projection rows
  int proj_stride;
  void* q_out;        // [T, H, D]
  void* k_cache;      // [NB, G, BS, D]
  void* v_cache;
  const int64_t* positions;
  const int64_t* slots;
  const float* cos_sin;  // [max_pos, rot_dims] = [cos | sin], or null
  int max_pos, rot_dims;
  const float* q_w;      // [H D]
  const float* k_w;      // [G D]
  const void* q_b;       // [H D] / [G D] of the projection's type, added to the q / k slices
  const void* k_b;       //   before anything else (the projection's biases), or null
  int T, H, G, D, BS, q_off, k_off;
  int64_t num_slots;     // NB * BS
  float eps;
};
void launch_proj_norm_rope_cache(const ProjParams& p, bool f32, hipStream_t s);

struct AttnParams {
  void* out;            // rows of out_stride elements; head h at columns [h D, (h+1) D)
  int out_stride;
  const void* q;        // [T, H, D]
  const void* k_cache;  // [NB, G, BS, D]
  const void* v_cache;
  const int32_t* block_tables;  // [B, max_blocks]
  int max_blocks;
  const int32_t* seq_lens;      // [B]
  const int32_t* q_start;       // [B + 1] (prefill)
  const int32_t* tile_seq;      // prefill tile map
  const int32_t* tile_row;
  int num_tiles, tile_rows;
  const void* gate;     // [T, H] logits with row stride gate_stride, or null
  int gate_stride;
  const float* sink;    // [H] or null
  float scale;
  int chunk, window;    // 0 = off
  int B, H, G, D, BS, NB;
  // decode split: partial (max, sum) [B, H, parts, 2] and outputs [B, H, parts, D]
  float* ws_ml;
  float* ws_o;
  int num_parts;
};
void launch_sink_attention_prefill(const AttnParams& p, bool f32, hipStream_t s);
void launch_sink_attention_decode(const AttnParams& p, bool f32, hipStream_t s);

// ---- grouped norms, token shift, latent attention, routed experts (latent.hip) ----------------
// x (fp32 rows of d) += y + bias + y2 (each may be null; y / bias of the activation type, y2
// fp32), then out1 = gnorm(x) * w1 and out2 = gnorm(x) * w2 (out2 / w2 may be null), the norm
// taken over `groups` equal consecutive parts of the row
// optional token shift of out1 inside the norm kernel, for batches whose every row is a sequence
// of its own with a distinct slot (decode steps): out1 = h + (state[slot] - h) * mu with h the
// normed row as stored (zeros for position 0), and state[slot] = h.  mu null: no shift.
struct ShiftArgs {
  const float* mu;       // [d]
  void* state;           // [slots, d] of out1's type
  const int32_t* slot;   // [rows]
  const int64_t* pos;    // [rows]
};
void launch_add_group_norm(void* out1, void* out2, bool out_f32, int out1_stride, int out2_stride,
                           float* x, const void* y, bool y_f32, int y_stride, const float* y2,
                           const void* bias, const float* w1, const float* w2, int rows, int d,
                           int groups, float eps, const ShiftArgs& sh, hipStream_t s);
// out[t] = h[t] + (prev - h[t]) * mu; then the last row of each sequence goes to state[slot].
// single: every row is a sequence of its own with a distinct slot (one launch instead of two)
void launch_token_shift(void* out, const void* h, const float* mu, void* state,
                        const int32_t* slot, const int64_t* pos, bool f32, int rows, int d,
                        bool single, hipStream_t s);

struct LatentPrepParams {
  const void* proj;   // [T, N] fused down-projection rows
  int proj_stride;
  void* cq_out;       // [T, q_rank]
  void* cache;        // [NB * BS, kv_rank + rot_dim] or null
  void* vgroups;      // [NB * BS / 8, kv_rank, 8]: the latent again, in 8-token groups, or null
  const int64_t* positions;
  const int64_t* slots;
  const float* cos_sin;  // [max_pos, rot_dim] = [cos | sin]
  int max_pos;
  const float* q_w;      // [q_rank]
  const float* kv_w;     // [kv_rank]
  int T, q_rank, kv_rank, rot_dim, q_off, kv_off;
  int64_t num_slots;
  float eps;
  int half_pairs;        // rotated pairs (i, i + rot_dim / 2) instead of (2i, 2i + 1)
};
void launch_latent_prep(const LatentPrepParams& p, bool f32, hipStream_t s);
// in place: `dims` entries from `offset` of each of the H heads (n entries per head) of a row; pairs
// (2i, 2i + 1), or (i, i + dims / 2) with half_pairs
void launch_rotate_heads(void* q, int q_stride, int T, int H, int n, int offset, int dims,
                         const int64_t* positions, const float* cos_sin, int max_pos, bool f32,
                         bool half_pairs, hipStream_t s);

struct LatentAttnParams {
  void* out;            // [H, T, R]
  const void* q_lat;    // [H, T, R]
  const void* q;        // [T, H, q_head]; the rotated part at rot_off of every head
  int q_stride, q_head, rot_off;
  const void* cache;    // [NB * BS, R + r]
  const int32_t* block_tables;  // [B, max_blocks]
  int max_blocks;
  const int32_t* seq_lens;      // [B]
  const int32_t* q_start;       // [B + 1], or null: row t is sequence t
  const int64_t* positions;     // [T]
  float scale;
  int T, B, H, R, r, BS;
  int vec;              // rows of the cache can be read in 16-byte pieces
  // matrix-core kernels only
  const void* vgroups;          // [NB * BS / 8, R, 8]
  int NB;
  const int32_t* tile_seq;      // prefill tile map: sequence and first chunk row of a tile
  const int32_t* tile_row;
  int num_tiles, tile_rows;
  float* ws_ml;                 // decode split: (max, sum) [B, H, parts, 2]
  float* ws_o;                  //               outputs    [B, H, parts, R]
  int num_parts;
};
void launch_latent_attention(const LatentAttnParams& p, bool f32, hipStream_t s);
// bf16, R / r among the built sizes (latent_mfma_sizes), BS % 32 == 0, 16-byte aligned rows
bool latent_mfma_sizes(int R, int r);
void launch_latent_prefill_mfma(const LatentAttnParams& p, hipStream_t s);
void launch_latent_decode_mfma(const LatentAttnParams& p, hipStream_t s);

// out [H, T, N] (strides o_hs / o_ts) = a [H, T, K] (strides a_hs / a_ts, unit in k) x
// w [H, N, K]^T, bf16, K % 16 == 0, N % 32 == 0, 16-byte aligned rows; meant for a few rows (one
// wave per 32 x 32 tile)
void launch_head_matmul(void* out, int64_t o_hs, int64_t o_ts, const void* a, int64_t a_hs,
                        int64_t a_ts, const void* w, int H, int T, int N, int K, hipStream_t s);
void launch_head_gate(void* out, int out_stride, const void* o, const void* gate, int gate_stride,
                      bool per_head, int rows, int H, int V, bool f32, hipStream_t s);
void launch_xielu(void* out, int out_stride, const void* x, int x_stride, const void* bias,
                  const float* act, int rows, int F, bool f32, hipStream_t s);
void launch_moe_route(int32_t* ids, float* w, const void* h, int h_stride, const float* router,
                      const float* corr, int rows, int d, int n, int top, int groups, int keep,
                      bool f32, hipStream_t s);
void launch_relu2_routed(void* out, int out_stride, const void* up, int up_stride,
                         const int32_t* ids, const float* w, int rows, int top, int E, int F,
                         bool f32, hipStream_t s);
void launch_moe_combine(float* out, const void* y, const int32_t* inv, const int32_t* ids,
                        const float* w, const void* h, int h_stride, int rows, int d, int top,
                        int E, int y_rows, bool f32, hipStream_t s);

// ---- sandwich norms, retention, head-mixed attention, logit-top-k routing (retention.hip) -------
// m = ya, or (rms(ya) wa + rms(yb) wb) / 2 when yb is given; x (fp32 rows of d) <- x + rms(m)
// post_w (fresh: x is not read); out = rms(x) next_w (next_w null: out = x).  Every weight has a stride of 1 (d
// entries) or 0 (one number).  ya / yb are both fp32 or both of the activation type.
void launch_post_norm_add_norm(void* out, bool out_f32, int out_stride, float* x, const void* ya,
                               int ya_stride, const void* yb, int yb_stride, bool y_f32,
                               const float* wa, int was, const float* wb, int wbs,
                               const float* post_w, int pws, const float* next_w, int nws,
                               int rows, int d, float eps, bool fresh, hipStream_t s);

struct HeadNormParams {
  const void* proj;   // [T, N] fused projection rows
  int proj_stride;
  void* q_out;        // [T, H, D]
  void* k_cache;      // [NB, G, BS, D]
  void* v_cache;      // [NB, G, BS / 8, Dv, 8]
  const int64_t* slots;
  int T, H, G, D, Dv, BS, q_off, k_off, v_off;
  int64_t num_slots;  // NB * BS
  float eps;
  bool norm_qk, norm_v;
  const float* q_w;   // [D] norm weights shared by the heads, or null
  const float* k_w;
  const float* cos_sin;       // [max_pos, rot_dims] = [cos | sin], rotate-half pairs, or null
  const int64_t* positions;   // [T] (with cos_sin)
  int max_pos, rot_dims;
};
void launch_head_norm_cache(const HeadNormParams& p, bool f32, hipStream_t s);

struct RetentionParams {
  void* out;            // rows of out_stride elements; head h at columns [h V, (h + 1) V)
  int out_stride;
  const void* proj;     // [T, N] fused projection rows
  int proj_stride;
  int q_off, k_off, v_off, g_off;
  float* state;         // [slots, H, V, D]: the transposed state of every slot and head
  int num_slots;
  const int32_t* seq_slot;   // [T]
  const int64_t* positions;  // [T]
  const int32_t* q_start;    // [num_seqs + 1] or null (row t is sequence t)
  const float* cos_sin;      // [max_pos, rot_dims] = [cos | sin] or null
  int rot_dims;
  const float* log2_decay;   // [H]
  int num_seqs, H, D, V;
  float eps;
  // segmented form (long prompt chunks, q_start given): states of the segments of SEG rows,
  // [num_segs, H, V, D] with num_segs = T / SEG + num_seqs; null: the direct form
  float* seg_buf;
  int SEG, num_segs;
  int DP, TC;           // set by the launcher
};
// 0 when the sizes do not fit a workgroup (ceil(V / 4) column groups x D / 32 lanes > 512)
int retention_dreg(int D, int V);
void launch_retention(RetentionParams p, bool f32, hipStream_t s);

struct TalkParams {
  void* out;            // rows of out_stride elements; head h at columns [h Dv, (h + 1) Dv)
  int out_stride;
  const void* q;        // [T, H, D]
  const void* k_cache;  // [NB, G, BS, D]
  const void* v_cache;  // [NB, G, BS / 8, Dv, 8]
  const int32_t* block_tables;  // [B, max_blocks]
  int max_blocks;
  const int32_t* seq_lens;      // [B]
  const int32_t* q_start;       // [B + 1] or null (row t is sequence t)
  const int64_t* positions;     // [T]
  const float* talk;    // [H, H] or null
  const void* gate;     // [T, H Dv] logits with row stride gate_stride, or null
  int gate_stride;
  float scale;
  int T, B, H, G, D, Dv, BS;
  // split form: (max, sum) [T, parts, H, 2] and unnormalised sums [T, parts, H, G Dv]
  float* ws_ml;
  float* ws_o;
  int num_parts;
  int row0;             // first row of a merge-only launch
};
size_t talking_attention_lds(int H, int D);
void launch_talking_attention(const TalkParams& p, bool f32, hipStream_t s);
void launch_talking_merge(const TalkParams& p, bool f32, hipStream_t s);
// matrix-core form for prompt chunks (bf16): fills the workspace of a one-partition split for
// the rows of the tile map (tile_seq / tile_row: sequence and first chunk row of a tile of
// tile_rows tokens, a multiple of 32); launch_talking_merge finishes
bool talk_mfma_supported(int H, int G, int D, int Dv, int BS);
// matrix-core form for one query per sequence (q_start null): fills the workspace of the
// num_parts-way split; launch_talking_merge finishes
void launch_talking_decode_mfma(const TalkParams& p, hipStream_t s);
void launch_talking_prefill_mfma(const TalkParams& p, const int32_t* tile_seq,
                                 const int32_t* tile_row, int num_tiles, int tile_rows,
                                 hipStream_t s);

void launch_route_topk(int32_t* ids, float* w, const void* h, int h_stride, const float* router,
                       const float* bias, int rows, int d, int n, int top, bool f32,
                       hipStream_t s);
// ids null: every weight is 1 (E = 1: a plain gated activation of [gate | up] rows)
// act 0: silu on the gate, 1: the tanh form of gelu
void launch_swiglu_routed(void* out, int out_stride, const void* gu, int gu_stride,
                          const int32_t* ids, const float* w, int rows, int top, int E, int F,
                          bool f32, int act, hipStream_t s);

// ---- several residual streams, state-space mixer, sigmoid group routing (hyper.hip) -----------
// xs [rows, S, d] fp32 in place: every stream from the old ones, xs_r <- sum_s mix[s, r] xs_s +
// w_out[r] (ya + yb + bias) (fresh: every stream <- fresh row); then u = sum_s w_in[s] xs_s and
// out = rmsnorm(u) * norm_w.  ya / yb rows of bf16 or fp32, each may be null.  S <= 8.
void launch_hyper_step(void* out, bool out_f32, int out_stride, float* xs, const float* fresh,
                       const void* ya, bool ya_f32, int ya_stride, const void* yb, bool yb_f32,
                       int yb_stride, const float* bias, const float* mix, const float* w_out,
                       const float* w_in, const float* norm_w, int rows, int S, int d, float eps,
                       hipStream_t s);
void launch_softcap(void* x, bool f32, size_t n, float cap, hipStream_t s);
// out = gnorm(y * silu(gate)) * w over `groups` equal parts of the n columns
void launch_gate_group_norm(void* out, int out_stride, const float* y, const void* gate,
                            int gate_stride, const float* w, bool f32, int rows, int n,
                            int groups, float eps, hipStream_t s);
// gates > 0: the router has that many rows after the E experts', whose sigmoids go to gate_w
// [rows, gates]
void launch_route_sigmoid(int32_t* ids, float* w, const void* h, int h_stride, bool f32,
                          const float* router, int rows, int d, int E, int top, int groups,
                          int keep, int group_top, float* gate_w, int gates, hipStream_t s);
// causal per-channel convolution of columns [off, off + C) of proj (b null: no bias; silu on the
// channels from silu_from on), then the sequences' last taps - 1 inputs to their slots; out fp32
// or proj's type; B sequences (q_start null: B = T, one row each)
void launch_conv_silu(void* out, bool out_f32, const void* proj, int proj_stride, int off, bool f32,
                      int silu_from, void* state, const float* w, const float* b, const int32_t* seq_slot,
                      const int64_t* positions, const int32_t* q_start, int T, int B, int C,
                      int taps, hipStream_t s);
// state rows a thread of the one-column scan keeps in registers (at most 64); can a head of V
// channels with N-entry states run (either form)?
int selective_scan_rows(int V, int N);
bool selective_scan_supported(int V, int N);
void launch_selective_scan(float* y, const float* xbc, const void* proj, int proj_stride,
                           int dt_off, bool f32, const float* dt_bias, const float* a_log,
                           const float* d_skip, float* state, const int32_t* seq_slot,
                           const int64_t* positions, const int32_t* q_start, int T, int B, int H,
                           int V, int N, int G, hipStream_t s);

// ---- matrix-state recurrences (recurrence.hip) ---------------------------------------------------
enum RecurrenceMode { kDecay = 0, kMatrixMemory = 1, kDelta = 2 };

struct RecurrenceParams {
  void* out;             // normed and gated heads, rows of out_stride; or
  int out_stride;
  float* raw;            // [T, H V]: the heads as they leave the state (raw given: out unused)
  const void* qkv;       // rows of qkv_stride: q, k (G heads of D) and v (H heads of V)
  int qkv_stride, q_off, k_off, v_off;
  int act;               // 1: silu on q, k and v
  const void* proj;      // rows of proj_stride: output gate, gates of the recurrence
  int proj_stride, g_off, a_off, b_off;
  const float* pa;       // [H] decay | forget gate bias | A_log
  const float* pb;       // [H] -     | input gate bias  | dt_bias
  float cap, q_scale, eps;
  float* state;          // [slots, H, V, D], transposed
  float* n_state;        // [slots, H, D] (matrix memory)
  float* m_state;        // [slots, H]
  int num_slots;
  const float* norm_w;   // [H V]
  int gate_act;          // 0 sigmoid, 1 silu
  const int32_t* seq_slot;
  const int64_t* positions;
  const int32_t* q_start;   // [num_seqs + 1] or null (row t is sequence t)
  int num_seqs, H, G, D, V;
  int VB, DP, TC;        // set by the launcher
};
// does a workgroup hold all state columns of a head (the head norm and gate can be fused)?
bool recurrence_fused(int D, int V);
bool recurrence_supported(int D, int V);
void launch_recurrence(RecurrenceParams p, int mode, bool f32, hipStream_t s);
// steps of single rows (q_start null), sizes, offsets and row strides in fours, 16-byte aligned
// rows; always holds a whole head
bool recurrence_step_supported(int D, int V);
void launch_recurrence_step(RecurrenceParams p, int mode, bool f32, hipStream_t s);
// chunked matrix-core form for prompt portions (recurrence_mfma.hip, bf16): the sequences of r
// (q_start given, pointing at the first chunked sequence, whose first row is row0); r.raw takes
// the heads as they leave the state (the matrix memory's still undivided, with den = n . q and
// floor = e^-m per row and head)
struct ChunkParams {
  RecurrenceParams r;
  int row0, num_chunks;   // chunk entries: rows / 64 + sequences
  float* la;              // [T, H] log decay / input scale (matrix memory only)
  float* lb;
  float* den;
  float* floor;
  // workspace, set by the launcher: operand fragments per (chunk, key head) and (chunk, head),
  // scalars per (chunk, head, token)
  uint16_t* qf;
  uint16_t* kf;
  uint16_t* ktf;
  uint16_t* pf;
  uint16_t* tf;
  float* sc;
  float* eend;            // e^(L_end) per (chunk, head)
};
bool chunk_supported(int D);
void chunk_workspace(int mode, int chunks, int H, int G, int D, int64_t* halves, int64_t* floats);
void launch_chunk_recurrence(ChunkParams p, int mode, uint16_t* halves, float* floats, hipStream_t s);
// out = gnorm(y / (max(|den|, floor) + 1e-6)) * w * act(gate) over `groups` equal parts of the n
// columns (den null: y itself; act 0 sigmoid, 1 silu)
void launch_norm_gate(void* out, int out_stride, const float* y, const void* gate, int gate_stride,
                      const float* w, const float* den, const float* floor, bool f32, int act,
                      int rows, int n, int groups, float eps, hipStream_t s);

// ---- window + pooled blocks attention (pooled_attention.hip) -----------------------------------
struct RopeCacheParams {
  const void* proj;      // [T, N] fused projection rows
  int proj_stride;
  void* q_out;           // [T, H, D]
  void* k_cache;         // [NB, G, BS, D]
  void* v_cache;         // [NB, G, BS / 8, Dv, 8]
  const int64_t* positions;
  const int64_t* slots;
  const float* cos_sin;  // [max_pos, rot_dims] = [cos | sin], or null
  const float* bias;     // [N] laid out like proj's columns, or null
  int max_pos, rot_dims;
  int T, H, G, D, Dv, BS, q_off, k_off, v_off;
  int64_t num_slots;
};
void launch_bias_rope_cache(const RopeCacheParams& p, bool f32, hipStream_t s);

struct PoolParams {
  const void* k_cache;
  const void* v_cache;
  float* k_pool;         // [NB, G, PS, D]
  float* v_pool;
  const int64_t* positions;
  const int64_t* slots;
  const int32_t* block_tables;
  const int32_t* q_start;   // [B + 1] or null
  int max_blocks, T, B, G, D, Dv, BS, PS, pool;
};
void launch_pool_cache_blocks(const PoolParams& p, bool f32, hipStream_t s);

struct PoolAttnParams {
  void* out;             // rows of out_stride; head h at columns [h Dv, (h + 1) Dv)
  int out_stride;
  const void* q;         // [T, H, D]
  const void* k_cache;
  const void* v_cache;
  const float* k_pool;   // or null (pool 0)
  const float* v_pool;
  const int32_t* block_tables;
  const int32_t* q_start;
  const int64_t* positions;
  const int64_t* slots;
  float scale;
  int max_blocks, T, B, H, G, D, Dv, BS, PS, window, pool, unit_sink;
};
void launch_pooled_window_attention(const PoolAttnParams& p, bool f32, hipStream_t s);
// matrix-core form for prompt chunks (bf16): the rows of the tile map (tile_seq / tile_row:
// sequence and first chunk row of a tile of 128 tokens)
bool pooled_mfma_supported(int H, int G, int D, int Dv, int BS);
void launch_pooled_window_prefill_mfma(const PoolAttnParams& p, const int32_t* tile_seq,
                                       const int32_t* tile_row, int num_tiles, hipStream_t s);
// matrix-core form for one query per sequence (row t = sequence t, the first `rows` rows): the
// query heads of a key/value head are the columns of a tile, the key range is split over the
// workgroup's waves
void launch_pooled_window_decode_mfma(const PoolAttnParams& p, int rows, hipStream_t s);

// ---- layer norms, clamped gated units, differential attention (diff.hip, diff_mfma.hip) --------
// m = ya + yb; x (fp32 rows of d) <- x + ln(m) post_w (fresh: x is not read; post_w null: m itself);
// out = ln(x) next_w (next_w null: out = x), ln over the row with the mean taken off
struct LayerNormStepParams {
  void* out;
  int out_stride;
  float* x;
  const void* ya;        // rows of bf16 or fp32
  int ya_stride, ya_f32;
  const void* yb;        // or null
  int yb_stride, yb_f32;
  const float* post_w;   // [d] or null
  const float* next_w;
  int rows, d, fresh;
  float eps;
};
void launch_layer_norm_step(const LayerNormStepParams& p, bool out_f32, hipStream_t s);

// out [rows, E F + Fs] from gu [rows, E 2F + 2 Fs] (per expert [gate | up], then the shared one):
// g' sigmoid(alpha g') (u' + 1), g' = min(c g, limit), u' = clamp(c u, -limit, limit), c the routing
// weight (0: not chosen; ids null: 1); the shared one times shared_w (null: 1)
struct ClampedGluParams {
  void* out;
  int out_stride;
  const void* gu;
  int gu_stride;
  const int32_t* ids;    // [rows, top] or null
  const float* w;
  const float* shared_w; // [rows] or null
  int rows, top, E, F, Fs;
  float limit, shared_limit, alpha;
};
void launch_clamped_glu(const ClampedGluParams& p, bool f32, hipStream_t s);

struct DiffAttnParams {
  void* out;             // rows of out_stride; head h at columns [h Dv, (h + 1) Dv)
  int out_stride;
  const void* q;         // rows of q_stride; head h at [h 2D, (h + 1) 2D): [map 1 | map 2]
  int q_stride;
  const void* k_cache;   // [NB, G, BS, 2 D]
  const void* v_cache;   // [NB, G, BS / 8, Dv, 8]
  const int32_t* block_tables;  // [B, max_blocks]
  int max_blocks;
  const int32_t* seq_lens;      // [B]
  const int32_t* q_start;       // [B + 1] or null (row t is sequence t)
  const int64_t* positions;     // [T] (row form)
  const int32_t* tile_seq;      // prefill tile map (matrix-core form)
  const int32_t* tile_row;
  int num_tiles, tile_rows;
  const void* gate;             // [T, H Dv] logits, or null
  int gate_stride;
  float lam, out_mult, scale, eps;   // out_mult: 1 - diff
  int chunk, T, B, H, G, D, Dv, BS, NB;
  // decode split: (max, sum) [B, H, 2, parts, 2] and unnormalised outputs [B, H, 2, parts, Dv]
  float* ws_ml;
  float* ws_o;
  int num_parts;
};
void launch_diff_attention(const DiffAttnParams& p, bool f32, hipStream_t s);
// bf16, sizes among the built ones, pages of a multiple of 32 keys
bool diff_mfma_supported(int D, int Dv, int BS);
void launch_diff_prefill_mfma(const DiffAttnParams& p, hipStream_t s);
void launch_diff_decode_mfma(const DiffAttnParams& p, hipStream_t s);

}  // namespace akap_stream
