// Matrix-core differential attention (bf16): two softmax maps per query head over the same values.
//
// v_mfma_f32_32x32x16_bf16 computes S^T = K Q^T (keys are the 32 rows, queries the 32 columns) and
// O^T = V^T P^T.  A query is a lane column: its softmax statistics are 16 registers and one
// exchange between the lane halves.  The K rows are loaded in the order (bits 2 and 3 of the row
// swapped) that makes a lane's S^T accumulators exactly the 8 keys of one value group, so P moves
// from accumulator to operand without lane traffic and the V^T operand is one 16-byte load from
// the cache [NB, G, BS / 8, Dv, 8].  A cached key is one row [map 1 | map 2] of 2 D entries.
//
// Prompt tiles: a wave owns 32 queries of one head under BOTH maps (two score tiles, two output
// accumulators), so every value fragment is loaded once for the two maps; the difference, the head
// norm, 1 - diff and the gate happen in registers (a query's output entries are the registers of
// two lanes).  Decode rows: the columns are up to 16 heads of one key/value head, under map 1 in
// the lower and under map 2 in the upper half of the tile; the score tile contracts over all 2 D
// entries of a key, the queries padded with zeros in the other map's half.  The key range is cut
// into partitions, one wave each, merged by a second launch.
#include "../kernels/common.h"
#include "stream.h"

namespace akap_stream {

using akap::bf16;
using akap::bf16x4;
using akap::bf16x8;
using akap::f32x16;

namespace {

constexpr float kLog2e = 1.44269504088896f;

__device__ __forceinline__ int swap23(int r) { return (r & ~12) | ((r & 4) << 1) | ((r & 8) >> 1); }

__device__ __forceinline__ int chunk_start(int pos, int chunk) {
  return chunk > 0 ? pos / chunk * chunk : 0;
}

// row of key j0 (a multiple of 32; pages are multiples of 32 keys) of key/value head g
__device__ __forceinline__ int key_row(const DiffAttnParams& p, const int32_t* bt, int g, int j0) {
  const int bi = j0 / p.BS;
  int blk = bi < p.max_blocks ? bt[bi] : 0;
  if (blk < 0 || blk >= p.NB) blk = 0;
  return (blk * p.G + g) * p.BS + (j0 - bi * p.BS);
}

// One 32-key block of one map: masks (unless every column sees the whole block), moves the running
// maximum (log2 units of the scaled scores) and sum, leaves the weights as B operands, rescales
// the outputs when a maximum moved.
template <int DVT>
__device__ __forceinline__ void softmax_block(f32x16& s, bf16x8 (&pb)[2], f32x16 (&o)[DVT], float& m,
                                              float& l, int j0, bool full, int pos, int lo,
                                              float sc2) {
  const int hf = (threadIdx.x & 63) >> 5;
  float bmax = -INFINITY;
  if (!full) {
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int key = j0 + 16 * (i >> 3) + 8 * hf + (i & 7);
      s[i] = key <= pos && key >= lo ? s[i] : -INFINITY;
    }
  }
#pragma unroll
  for (int i = 0; i < 16; ++i) bmax = fmaxf(bmax, s[i]);
  bmax = fmaxf(bmax, __shfl_xor(bmax, 32, 64));
  const float mn = fmaxf(m, bmax * sc2);
  const float ms = mn == -INFINITY ? 0.f : mn;       // nothing visible yet: every weight below is 0
  const float alpha = __builtin_amdgcn_exp2f(m - ms);
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    const float w = __builtin_amdgcn_exp2f(fmaf(s[i], sc2, -ms));
    sum += w;
    pb[i >> 3][i & 7] = (bf16)w;
  }
  sum += __shfl_xor(sum, 32, 64);
  l = l * alpha + sum;
  m = mn;
  if (__any(alpha != 1.0f)) {                        // (wave-uniform) the maxima settle early
#pragma unroll
    for (int k = 0; k < DVT; ++k)
#pragma unroll
      for (int i = 0; i < 16; ++i) o[k][i] *= alpha;
  }
}

// 1 / rms of a head's difference v (registers of this lane, its other half and, for split heads,
// `other`: the share of the wave that holds the rest) times 1 - diff
template <int DVT>
__device__ __forceinline__ float sum_squares(const f32x16 (&v)[DVT]) {
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < DVT; ++k)
#pragma unroll
    for (int i = 0; i < 16; ++i) ss += v[k][i] * v[k][i];
  return ss + __shfl_xor(ss, 32, 64);
}

// scale, gate, store DVT tiles of head h from value entry d0 on.  Register i of tile k: entry
// d0 + 32 k + 8 (i >> 2) + 4 hf + (i & 3).
template <int DVT>
__device__ __forceinline__ void store_head(const f32x16 (&v)[DVT], float ss, const DiffAttnParams& p,
                                           int t, int h, int d0) {
  const int hf = (threadIdx.x & 63) >> 5;
  const float f = p.out_mult / sqrtf(ss / (float)p.Dv + p.eps);
  const size_t c = (size_t)h * p.Dv + d0 + 4 * hf;
  bf16* o = (bf16*)p.out + (size_t)t * p.out_stride + c;
  const bf16* gt = p.gate ? (const bf16*)p.gate + (size_t)t * p.gate_stride + c : nullptr;
#pragma unroll
  for (int k = 0; k < DVT; ++k)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      bf16x4 r;
      bf16x4 gv;
      if (gt) gv = *(const bf16x4*)(gt + 32 * k + 8 * j);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float a = v[k][4 * j + i] * f;
        if (gt) a *= 1.0f / (1.0f + __expf(-(float)gv[i]));
        r[i] = (bf16)a;
      }
      *(bf16x4*)(o + 32 * k + 8 * j) = r;
    }
}

// Flat grid: (tile of 128 tokens, key/value head) units dealt over the XCDs longest first, the
// query heads of a unit are consecutive workgroups of ONE XCD; 32 queries per wave.  SPLIT 2: two
// waves share a query tile, each with half of the value entries (DVT tiles of 32 per wave), so
// that wide values fit the registers; both compute the scores.  The maps take turns (one score
// tile and one map's K fragments live at a time, the queries in LDS), which leaves room for two
// waves per SIMD: the fragments of map 2 are requested ahead of map 1's softmax, those of the next
// block's map 1 ahead of map 2's, the V fragments at the start of the block.
template <int KS, int DVT, int SPLIT>
__global__ __launch_bounds__(256 * SPLIT, 2) void diff_prefill_mfma_kernel(DiffAttnParams p) {
  constexpr int D = 16 * KS, Dv = 32 * DVT * SPLIT;
  __shared__ bf16x8 qs_all[4][2 * KS][64];           // [query tile][map, step][lane]
  __shared__ float share[4 * SPLIT][32];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int qt = wave / SPLIT, d0 = (wave % SPLIT) * 32 * DVT;
  const int col = lane & 31, hf = lane >> 5;
  const int rep = p.H / p.G;
  const int xcd = blockIdx.x & 7, jx = blockIdx.x >> 3;
  const int unit = (jx / rep) * 8 + xcd;
  if (unit >= p.num_tiles * p.G) return;             // (workgroup-uniform, like the next two)
  const int tile = p.num_tiles - 1 - unit / p.G;     // the map is sorted by rising work
  const int g = unit % p.G, h = g * rep + jx % rep;
  const int b = p.tile_seq[tile];
  if (b < 0 || b >= p.B) return;
  const int qs0 = p.q_start[b];
  const int qlen = p.q_start[b + 1] - qs0;
  const int kv = p.seq_lens[b];
  if (kv < qlen) return;
  const int rend = min(p.tile_row[tile] + p.tile_rows, qlen);
  const float sc2 = p.scale * kLog2e;
  const int32_t* bt = p.block_tables + (size_t)b * p.max_blocks;
  const bf16* kc = (const bf16*)p.k_cache;
  const bf16* vc = (const bf16*)p.v_cache;
  const int krow = swap23(col);
  const int r0 = p.tile_row[tile] + qt * 32;
  const bool active = r0 < rend;                     // the others only meet the barriers
  const int r = r0 + col;
  const bool valid = r < rend;
  const int t = qs0 + (valid ? r : active ? r0 : 0);
  const int pos = kv - qlen + r;
  const int lo = chunk_start(pos, p.chunk);
  bf16x8 (&qs)[2 * KS][64] = qs_all[qt];
  if (wave % SPLIT == 0) {
    const bf16* qp = (const bf16*)p.q + (size_t)t * p.q_stride + (size_t)h * 2 * D + 8 * hf;
#pragma unroll
    for (int c = 0; c < 2 * KS; ++c) qs[c][lane] = *(const bf16x8*)(qp + 16 * c);
  }
  __syncthreads();
  // the wave's range; columns past the tile's end compute like real ones and are not stored
  const int first = kv - qlen + r0;
  const int end = active ? kv - qlen + min(r0 + 31, rend - 1) : -1;
  const int lo_last = chunk_start(first + 31, p.chunk);
  const int jb = active ? chunk_start(first, p.chunk) & ~31 : 0;
  f32x16 o[2][DVT];
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int k = 0; k < 2; ++k)
#pragma unroll
    for (int d = 0; d < DVT; ++d)
#pragma unroll
      for (int i = 0; i < 16; ++i) o[k][d][i] = 0.f;

  if (active) {
    int row0 = key_row(p, bt, g, jb);
    int row1 = jb + 32 <= end ? key_row(p, bt, g, jb + 32) : 0;
    bf16x8 kf[KS];
    auto load_k = [&](int row, int map) {
      const bf16* kp = kc + ((size_t)row + krow) * (2 * D) + map * D + 8 * hf;
#pragma unroll
      for (int c = 0; c < KS; ++c) kf[c] = *(const bf16x8*)(kp + 16 * c);
    };
    load_k(row0, 0);
    for (int j0 = jb; j0 <= end; j0 += 32) {
      const bf16* vp = vc + (((size_t)(row0 >> 3) + hf) * Dv + d0 + col) * 8;
      bf16x8 vf[DVT][2];
      auto load_v = [&] {
#pragma unroll
        for (int d = 0; d < DVT; ++d)
#pragma unroll
          for (int sl = 0; sl < 2; ++sl)
            vf[d][sl] = *(const bf16x8*)(vp + ((size_t)(2 * sl) * Dv + 32 * d) * 8);
      };
      if (KS <= 4) load_v();
      const bool full = j0 + 31 <= first && j0 >= lo_last;
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        f32x16 s;
#pragma unroll
        for (int i = 0; i < 16; ++i) s[i] = 0.f;
#pragma unroll
        for (int c = 0; c < KS; ++c)
          s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[c], qs[k * KS + c][lane], s, 0, 0, 0);
        if (k == 0) {
          if (KS > 4) {                              // long rows: not beside the score products
            __builtin_amdgcn_sched_barrier(0);
            load_v();
          }
          load_k(row0, 1);
        } else if (j0 + 32 <= end) {
          row0 = row1;
          load_k(row0, 0);
          if (j0 + 64 <= end) row1 = key_row(p, bt, g, j0 + 64);
        }
        bf16x8 pb[2];
        softmax_block<DVT>(s, pb, o[k], m[k], l[k], j0, full, pos, lo, sc2);
#pragma unroll
        for (int d = 0; d < DVT; ++d)
#pragma unroll
          for (int sl = 0; sl < 2; ++sl)
            o[k][d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[d][sl], pb[sl], o[k][d], 0, 0, 0);
      }
    }
  }
  const float f1 = l[0] > 0.f ? 1.0f / l[0] : 0.f, f2 = l[1] > 0.f ? p.lam / l[1] : 0.f;
#pragma unroll
  for (int d = 0; d < DVT; ++d)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[0][d][i] = o[0][d][i] * f1 - o[1][d][i] * f2;
  float ss = sum_squares<DVT>(o[0]);
  if constexpr (SPLIT > 1) {
    if (hf == 0) share[wave][col] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int k = 0; k < SPLIT; ++k) ss += share[qt * SPLIT + k][col];
  }
  if (valid) store_head<DVT>(o[0], ss, p, t, h, d0);
}

// grid (B, G * ceil(rep / 16), parts), one wave
template <int KS, int DVT>
__global__ __launch_bounds__(64) void diff_decode_mfma_kernel(DiffAttnParams p) {
  constexpr int D = 16 * KS, Dv = 32 * DVT;
  const int lane = threadIdx.x;
  const int col = lane & 31, hf = lane >> 5;
  const int map = col >> 4;
  const int rep = p.H / p.G, cg = (rep + 15) >> 4;
  const int b = blockIdx.x, g = blockIdx.y / cg, part = blockIdx.z;
  const int hc = (blockIdx.y % cg) * 16 + (col & 15);
  const bool valid = hc < rep;
  const int h = g * rep + (valid ? hc : 0);
  const int kv = p.seq_lens[b];
  if (kv <= 0) {                                     // a padding row: defined output
    if (part == 0 && valid && map == 0) {
      bf16* o = (bf16*)p.out + (size_t)b * p.out_stride + (size_t)h * Dv;
      for (int d = hf; d < Dv; d += 2) o[d] = (bf16)0.f;
    }
    return;
  }
  const int pos = kv - 1, lo = chunk_start(pos, p.chunk), a0 = lo & ~31;
  int per = (pos + 1 - a0 + p.num_parts - 1) / p.num_parts;
  per = (per + 31) & ~31;
  const int jb = a0 + part * per, je = min(pos, jb + per - 1);
  const float sc2 = p.scale * kLog2e;
  const int32_t* bt = p.block_tables + (size_t)b * p.max_blocks;
  // the query under the lane's map, zeros under the other one
  bf16x8 qf[2 * KS];
  {
    const bf16* qp = (const bf16*)p.q + (size_t)b * p.q_stride + (size_t)h * 2 * D + 8 * hf;
#pragma unroll
    for (int c = 0; c < 2 * KS; ++c) {
      qf[c] = *(const bf16x8*)(qp + 16 * c);
      if ((c >= KS ? 1 : 0) != map) {
#pragma unroll
        for (int i = 0; i < 8; ++i) qf[c][i] = (bf16)0.f;
      }
    }
  }
  f32x16 o[DVT];
  float m = -INFINITY, l = 0.f;
#pragma unroll
  for (int d = 0; d < DVT; ++d)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[d][i] = 0.f;
  if (jb <= je) {
    const int krow = swap23(col);
    int row0 = key_row(p, bt, g, jb);
    int row1 = jb + 32 <= je ? key_row(p, bt, g, jb + 32) : 0;
    bf16x8 kf[2 * KS];
    auto load_k = [&](int row) {
      const bf16* kp = (const bf16*)p.k_cache + ((size_t)row + krow) * (2 * D) + 8 * hf;
#pragma unroll
      for (int c = 0; c < 2 * KS; ++c) kf[c] = *(const bf16x8*)(kp + 16 * c);
    };
    load_k(row0);
    for (int j0 = jb; j0 <= je; j0 += 32) {
      const bf16* vp = (const bf16*)p.v_cache + (((size_t)(row0 >> 3) + hf) * Dv + col) * 8;
      bf16x8 vf[DVT][2];
#pragma unroll
      for (int d = 0; d < DVT; ++d)
#pragma unroll
        for (int sl = 0; sl < 2; ++sl)
          vf[d][sl] = *(const bf16x8*)(vp + ((size_t)(2 * sl) * Dv + 32 * d) * 8);
      f32x16 s;
#pragma unroll
      for (int i = 0; i < 16; ++i) s[i] = 0.f;
#pragma unroll
      for (int c = 0; c < 2 * KS; ++c)
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[c], qf[c], s, 0, 0, 0);
      if (j0 + 32 <= je) {
        row0 = row1;
        load_k(row0);
        if (j0 + 64 <= je) row1 = key_row(p, bt, g, j0 + 64);
      }
      bf16x8 pb[2];
      softmax_block<DVT>(s, pb, o, m, l, j0, j0 + 31 <= pos && j0 >= lo, pos, lo, sc2);
#pragma unroll
      for (int d = 0; d < DVT; ++d)
#pragma unroll
        for (int sl = 0; sl < 2; ++sl)
          o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[d][sl], pb[sl], o[d], 0, 0, 0);
    }
  }
  if (p.num_parts > 1) {
    if (!valid) return;
    const size_t slot = (((size_t)b * p.H + h) * 2 + map) * p.num_parts + part;
    if (hf == 0) {
      p.ws_ml[slot * 2] = m;
      p.ws_ml[slot * 2 + 1] = l;
    }
#pragma unroll
    for (int d = 0; d < DVT; ++d)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        *(float4*)(p.ws_o + slot * Dv + 32 * d + 8 * j + 4 * hf) =
            make_float4(o[d][4 * j], o[d][4 * j + 1], o[d][4 * j + 2], o[d][4 * j + 3]);
    return;
  }
  // map 2 of a head sits 16 columns above map 1
  const float f = l > 0.f ? (map ? p.lam : 1.0f) / l : 0.f;
#pragma unroll
  for (int d = 0; d < DVT; ++d)
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const float a = o[d][i] * f;
      o[d][i] = a - __shfl_xor(a, 16, 64);
    }
  const float ss = sum_squares<DVT>(o);
  if (valid && map == 0) store_head<DVT>(o, ss, p, b, h, 0);
}

// grid (B, H), 128 threads: the partitions of one (row, head) under both maps
__global__ __launch_bounds__(128) void diff_decode_merge_kernel(DiffAttnParams p) {
  __shared__ float wts[2][64];                       // weight of every partition over the map's sum
  __shared__ float scratch[16];
  const int b = blockIdx.x, h = blockIdx.y, np = p.num_parts, Dv = p.Dv;
  if (p.seq_lens[b] <= 0) return;                    // the partition kernel zeroed the row
  const size_t base = ((size_t)b * p.H + h) * 2 * np;
  {
    // wave k: map k, a partition per lane (at most 64)
    const int k = threadIdx.x >> 6, i = threadIdx.x & 63;
    const float mi = i < np ? p.ws_ml[(base + k * np + i) * 2] : -INFINITY;
    const float li = i < np ? p.ws_ml[(base + k * np + i) * 2 + 1] : 0.f;
    const float mm = akap::wave_max(li > 0.f ? mi : -INFINITY);
    const float w = li > 0.f ? __builtin_amdgcn_exp2f(mi - mm) : 0.f;
    const float l = akap::wave_sum(li * w);
    wts[k][i] = l > 0.f ? w * (k ? -p.lam : 1.0f) / l : 0.f;
  }
  __syncthreads();
  float v[2] = {0.f, 0.f};                           // entries threadIdx.x and + 128
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int d = threadIdx.x + 128 * c;
    if (d < Dv)
      for (int k = 0; k < 2; ++k)
        for (int i = 0; i < np; ++i)
          if (wts[k][i] != 0.f) v[c] += p.ws_o[(base + k * np + i) * Dv + d] * wts[k][i];
  }
  const float ss = akap::block_sum(v[0] * v[0] + v[1] * v[1], scratch);
  const float f = p.out_mult / sqrtf(ss / (float)Dv + p.eps);
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int d = threadIdx.x + 128 * c;
    if (d < Dv) {
      float a = v[c] * f;
      if (p.gate)
        a *= 1.0f / (1.0f + __expf(-(float)((const bf16*)p.gate)[(size_t)b * p.gate_stride + (size_t)h * Dv + d]));
      ((bf16*)p.out)[(size_t)b * p.out_stride + (size_t)h * Dv + d] = (bf16)a;
    }
  }
}

}  // namespace

// (query/key size, value size) pairs the kernels are built for
#define DIFF_SIZES(F)                                \
  F(16, 32) F(16, 64) F(32, 32) F(32, 64) F(32, 128) \
  F(64, 64) F(64, 128) F(64, 256) F(128, 128) F(128, 256)

bool diff_mfma_supported(int D, int Dv, int BS) {
  if (BS % 32) return false;
#define F(a, c) if (D == a && Dv == c) return true;
  DIFF_SIZES(F)
#undef F
  return false;
}

void launch_diff_prefill_mfma(const DiffAttnParams& p, hipStream_t s) {
  if (p.num_tiles <= 0) return;
  const unsigned grid = (unsigned)((p.num_tiles * p.G + 7) / 8 * 8) * (p.H / p.G);
#define F(a, c)                                                                       \
  if (p.D == a && p.Dv == c) {                                                        \
    constexpr int sp = c > 128 ? 2 : 1;                                               \
    diff_prefill_mfma_kernel<a / 16, c / 32 / sp, sp><<<grid, 256 * sp, 0, s>>>(p);   \
  }
  DIFF_SIZES(F)
#undef F
}

void launch_diff_decode_mfma(const DiffAttnParams& p, hipStream_t s) {
  if (p.B <= 0) return;
  const int rep = p.H / p.G;
  const dim3 grid(p.B, p.G * ((rep + 15) / 16), p.num_parts);
#define F(a, c) \
  if (p.D == a && p.Dv == c) diff_decode_mfma_kernel<a / 16, c / 32><<<grid, 64, 0, s>>>(p);
  DIFF_SIZES(F)
#undef F
  if (p.num_parts > 1) diff_decode_merge_kernel<<<dim3(p.B, p.H), 128, 0, s>>>(p);
}

}  // namespace akap_stream
