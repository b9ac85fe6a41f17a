// Kernels of layers with layer norms around every sublayer, differential attention and clamped
// gated experts: post layer norm + residual + next layer norm, the clamped gated unit with the
// routing weight on its input, and the row form of the differential attention (any head size,
// bf16 and fp32; the matrix-core form is in diff_mfma.hip).
//
// Means, variances, scores, softmax, the difference of the two maps, its norm, gates and the
// residual sum are fp32 whatever the storage type; every size is a run-time argument.
#include "../kernels/common.h"
#include "stream.h"

namespace akap_stream {

using akap::bf16;
using akap::block_sum;
using akap::wave_max;
using akap::wave_sum;

namespace {

template <typename T>
__device__ __forceinline__ float ldf(const T* p) { return (float)*p; }

__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + __expf(-z)); }

// 8 consecutive elements (32- resp. 16-byte aligned) as floats, and back
__device__ __forceinline__ void ld8(const float* p, float (&v)[8]) {
  const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
  v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void ld8(const bf16* p, float (&v)[8]) {
  const akap::bf16x8 a = *(const akap::bf16x8*)p;
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = (float)a[i];
}
__device__ __forceinline__ void st8(float* p, const float (&v)[8]) {
  *(float4*)p = make_float4(v[0], v[1], v[2], v[3]);
  *(float4*)(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
}
__device__ __forceinline__ void st8(bf16* p, const float (&v)[8]) {
  akap::bf16x8 o;
#pragma unroll
  for (int i = 0; i < 8; ++i) o[i] = (bf16)v[i];
  *(akap::bf16x8*)p = o;
}

// ------------------------------------------------------------------ layer norms around a sublayer
// One workgroup per row, the row in registers: NR pieces of 8 columns per thread.  The addends are
// bf16 or fp32 each (workgroup-uniform switches).
template <typename TO, int NR>
__global__ __launch_bounds__(256) void layer_norm_step_vec_kernel(LayerNormStepParams p) {
  __shared__ float scratch[16];
  const int row = blockIdx.x, d = p.d;
  float v[NR][8];
  float sum = 0.f;
#pragma unroll
  for (int k = 0; k < NR; ++k) {
    const int c = (k * 256 + threadIdx.x) * 8;
    if (c >= d) {
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] = 0.f;
      continue;
    }
    if (p.ya_f32) ld8((const float*)p.ya + (size_t)row * p.ya_stride + c, v[k]);
    else ld8((const bf16*)p.ya + (size_t)row * p.ya_stride + c, v[k]);
    if (p.yb) {
      float b[8];
      if (p.yb_f32) ld8((const float*)p.yb + (size_t)row * p.yb_stride + c, b);
      else ld8((const bf16*)p.yb + (size_t)row * p.yb_stride + c, b);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] += b[i];
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) sum += v[k][i];
  }
  const float inv_d = 1.0f / (float)d;
  // (v - mean) / sqrt(var + eps), two passes over the registers
  auto stats = [&](float s, float& mean, float& rstd) {
    mean = block_sum(s, scratch) * inv_d;
    float q = 0.f;
#pragma unroll
    for (int k = 0; k < NR; ++k)
      if ((k * 256 + (int)threadIdx.x) * 8 < d)
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const float e = v[k][i] - mean;
          q += e * e;
        }
    rstd = 1.0f / sqrtf(block_sum(q, scratch) * inv_d + p.eps);
  };
  float mean = 0.f, rstd = 1.f;
  if (p.post_w) stats(sum, mean, rstd);
  float* xr = p.x + (size_t)row * d;
  sum = 0.f;
#pragma unroll
  for (int k = 0; k < NR; ++k) {
    const int c = (k * 256 + threadIdx.x) * 8;
    if (c >= d) continue;
    if (p.post_w) {
      float w[8];
      ld8(p.post_w + c, w);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] = (v[k][i] - mean) * rstd * w[i];
    }
    if (!p.fresh) {
      float x[8];
      ld8(xr + c, x);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] += x[i];
    }
    st8(xr + c, v[k]);
#pragma unroll
    for (int i = 0; i < 8; ++i) sum += v[k][i];
  }
  mean = 0.f;
  rstd = 1.f;
  if (p.next_w) stats(sum, mean, rstd);
  TO* o = (TO*)p.out + (size_t)row * p.out_stride;
#pragma unroll
  for (int k = 0; k < NR; ++k) {
    const int c = (k * 256 + threadIdx.x) * 8;
    if (c >= d) continue;
    if (p.next_w) {
      float w[8];
      ld8(p.next_w + c, w);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] = (v[k][i] - mean) * rstd * w[i];
    }
    st8(o + c, v[k]);
  }
}

// any row length up to the LDS; a thread keeps to its own columns in every phase
template <typename TO>
__global__ __launch_bounds__(256) void layer_norm_step_kernel(LayerNormStepParams p) {
  extern __shared__ float r[];
  __shared__ float scratch[16];
  const int row = blockIdx.x, d = p.d;
  const float inv_d = 1.0f / (float)d;
  auto at = [&](const void* y, int f32, int stride, int c) {
    return f32 ? ((const float*)y)[(size_t)row * stride + c]
               : (float)((const bf16*)y)[(size_t)row * stride + c];
  };
  float sum = 0.f;
  for (int c = threadIdx.x; c < d; c += 256) {
    float f = at(p.ya, p.ya_f32, p.ya_stride, c);
    if (p.yb) f += at(p.yb, p.yb_f32, p.yb_stride, c);
    r[c] = f;
    sum += f;
  }
  auto stats = [&](float s, float& mean, float& rstd) {
    mean = block_sum(s, scratch) * inv_d;
    float q = 0.f;
    for (int c = threadIdx.x; c < d; c += 256) {
      const float e = r[c] - mean;
      q += e * e;
    }
    rstd = 1.0f / sqrtf(block_sum(q, scratch) * inv_d + p.eps);
  };
  float mean = 0.f, rstd = 1.f;
  if (p.post_w) stats(sum, mean, rstd);
  float* xr = p.x + (size_t)row * d;
  sum = 0.f;
  for (int c = threadIdx.x; c < d; c += 256) {
    float f = r[c];
    if (p.post_w) f = (f - mean) * rstd * p.post_w[c];
    if (!p.fresh) f += xr[c];
    xr[c] = f;
    r[c] = f;
    sum += f;
  }
  mean = 0.f;
  rstd = 1.f;
  if (p.next_w) stats(sum, mean, rstd);
  TO* o = (TO*)p.out + (size_t)row * p.out_stride;
  for (int c = threadIdx.x; c < d; c += 256)
    o[c] = (TO)(p.next_w ? (r[c] - mean) * rstd * p.next_w[c] : r[c]);
}

// ------------------------------------------------------------------ clamped gated units
__device__ __forceinline__ float clamped_unit(float g, float u, float limit, float alpha) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * (1.0f / (1.0f + __expf(-alpha * g))) * (u + 1.0f);
}

// grid (rows, column blocks); W columns per thread (8: sizes, strides and pointers allow 16-byte
// accesses and no piece of 8 crosses an expert)
template <typename T, int W>
__global__ __launch_bounds__(256) void clamped_glu_kernel(ClampedGluParams p) {
  const int t = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * W;
  const int n0 = p.E * p.F;
  if (c >= n0 + p.Fs) return;
  const T* g = (const T*)p.gu + (size_t)t * p.gu_stride;
  T* o = (T*)p.out + (size_t)t * p.out_stride + c;
  float in = 1.f, outw = 1.f, limit = p.limit;
  int F = p.F;
  if (c < n0) {
    const int e = c / p.F;
    g += (size_t)e * 2 * p.F + (c - e * p.F);
    if (p.ids) {
      in = 0.f;
      for (int k = 0; k < p.top; ++k)
        if (p.ids[(size_t)t * p.top + k] == e) in = p.w[(size_t)t * p.top + k];
    }
  } else {
    g += (size_t)2 * n0 + (c - n0);
    F = p.Fs;
    limit = p.shared_limit;
    if (p.shared_w) outw = p.shared_w[t];
  }
  if constexpr (W == 8) {
    float a[8], b[8];
    if (in == 0.f) {          // not chosen: the unit of a zero input is zero
#pragma unroll
      for (int i = 0; i < 8; ++i) a[i] = 0.f;
    } else {
      ld8(g, a);
      ld8(g + F, b);
#pragma unroll
      for (int i = 0; i < 8; ++i) a[i] = outw * clamped_unit(in * a[i], in * b[i], limit, p.alpha);
    }
    st8(o, a);
  } else {
    *o = (T)(in == 0.f ? 0.f
                       : outw * clamped_unit(in * ldf(g), in * ldf(g + F), limit, p.alpha));
  }
}

// ------------------------------------------------------------------ differential attention, rows
// One wave per (token, query head), the 4 waves of a workgroup take 4 heads of one token.  Keys go
// in 64-aligned pieces: a lane scores one key under both maps (a cached key is one row of 2 D
// entries), the wave takes each map's maximum and sum, then lanes own output entries and read the
// values once for both maps, one 8-key group at a time.
template <typename T>
__device__ __forceinline__ float dot_part(const float* q, const T* k, int n) {
  float s = 0.f;
  constexpr int W = 16 / (int)sizeof(T);
  int d = 0;
  if (((uintptr_t)k & 15) == 0)
    for (; d + W <= n; d += W) {
      float v[W];
      if constexpr (sizeof(T) == 2) {
        const akap::bf16x8 x = *(const akap::bf16x8*)(k + d);
#pragma unroll
        for (int e = 0; e < W; ++e) v[e] = (float)x[e];
      } else {
        const akap::f32x4 x = *(const akap::f32x4*)(k + d);
#pragma unroll
        for (int e = 0; e < W; ++e) v[e] = x[e];
      }
#pragma unroll
      for (int e = 0; e < W; ++e) s += q[d + e] * v[e];
    }
  for (; d < n; ++d) s += q[d] * ldf(k + d);
  return s;
}

__device__ __forceinline__ void ld_group(float (&v)[8], const bf16* p) { ld8(p, v); }
__device__ __forceinline__ void ld_group(float (&v)[8], const float* p) { ld8(p, v); }

template <typename T, int NR>
__global__ __launch_bounds__(256) void diff_attention_kernel(DiffAttnParams p) {
  extern __shared__ float lds[];
  const int t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int h = blockIdx.y * 4 + wave;
  int b = t;
  if (p.q_start != nullptr) {
    int lo = 0, hi = p.B - 1;
    while (lo < hi) {
      const int mid = (lo + hi + 1) >> 1;
      if (p.q_start[mid] <= t) lo = mid; else hi = mid - 1;
    }
    b = lo;
    if (t >= p.q_start[p.B]) return;
  }
  if (h >= p.H) return;                              // uniform per wave; no barriers below
  const int kv = p.seq_lens[b];
  const int D = p.D, Dv = p.Dv, BS = p.BS;
  T* o = (T*)p.out + (size_t)t * p.out_stride + (size_t)h * Dv;
  if (kv <= 0) {                                     // a padding row: defined output
    for (int d = lane; d < Dv; d += 64) o[d] = (T)0.f;
    return;
  }
  const int64_t pos = p.positions[t];
  const int last = (int)(pos < kv ? pos : kv - 1);
  const int lo = p.chunk > 0 ? last / p.chunk * p.chunk : 0;
  float* q = lds + wave * (2 * D + 128);             // [map 1 | map 2], scaled
  float* ps = q + 2 * D;                             // weights of a piece, [2][64]
  const T* qg = (const T*)p.q + (size_t)t * p.q_stride + (size_t)h * 2 * D;
  for (int c = lane; c < 2 * D; c += 64) q[c] = ldf(qg + c) * p.scale;
  __builtin_amdgcn_wave_barrier();
  const int g = h / (p.H / p.G), NG = BS >> 3;
  const int32_t* bt = p.block_tables + (size_t)b * p.max_blocks;
  float acc[2][NR], m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int k = 0; k < 2; ++k)
#pragma unroll
    for (int i = 0; i < NR; ++i) acc[k][i] = 0.f;
  for (int base = lo & ~63; base <= last; base += 64) {
    const int j = base + lane;
    const bool ok = j >= lo && j <= last;
    int grow = 0;
    float s[2] = {-INFINITY, -INFINITY};
    if (j <= last) {
      const int bi = j / BS;
      int blk = bi < p.max_blocks ? bt[bi] : 0;
      if (blk < 0 || blk >= p.NB) blk = 0;
      const int off = j - bi * BS;
      grow = (blk * p.G + g) * NG + (off >> 3);
      if (ok) {
        const T* kr = (const T*)p.k_cache + ((size_t)(blk * p.G + g) * BS + off) * 2 * D;
        s[0] = dot_part(q, kr, D);
        s[1] = dot_part(q + D, kr + D, D);
      }
    }
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const float mn = fmaxf(m[k], wave_max(s[k]));  // finite: a piece always holds a visible key
      const float corr = expf(m[k] - mn);            // first piece: exp(-inf) = 0
      const float pj = ok ? expf(s[k] - mn) : 0.f;
      l[k] = l[k] * corr + wave_sum(pj);
      m[k] = mn;
      ps[k * 64 + lane] = pj;
#pragma unroll
      for (int i = 0; i < NR; ++i) acc[k][i] *= corr;
    }
    __builtin_amdgcn_wave_barrier();
    for (int gi = 0; gi < 8; ++gi) {
      const int gb = base + gi * 8;
      if (gb > last || gb + 8 <= lo) continue;       // (wave-uniform) nothing visible in the group
      const int gr = __shfl(grow, gi * 8, 64);
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        const int d = i * 64 + lane;
        if (d < Dv) {
          float v[8];
          ld_group(v, (const T*)p.v_cache + ((size_t)gr * Dv + d) * 8);
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            acc[0][i] += ps[gi * 8 + e] * v[e];
            acc[1][i] += ps[64 + gi * 8 + e] * v[e];
          }
        }
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
  const float f1 = 1.0f / l[0], f2 = p.lam / l[1];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const float a = i * 64 + lane < Dv ? acc[0][i] * f1 - acc[1][i] * f2 : 0.f;
    acc[0][i] = a;
    ss += a * a;
  }
  ss = wave_sum(ss);
  const float f = p.out_mult / sqrtf(ss / (float)Dv + p.eps);
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int d = i * 64 + lane;
    if (d < Dv) {
      float a = acc[0][i] * f;
      if (p.gate) a *= sigmoidf(ldf((const T*)p.gate + (size_t)t * p.gate_stride + (size_t)h * Dv + d));
      o[d] = (T)a;
    }
  }
}

bool aligned(const void* p, size_t a) { return p == nullptr || ((uintptr_t)p % a) == 0; }

}  // namespace

// ================================================================== launchers
void launch_layer_norm_step(const LayerNormStepParams& p, bool out_f32, hipStream_t s) {
  if (p.rows <= 0) return;
  const bool vec = p.d % 8 == 0 && p.d <= 8192 && p.out_stride % 8 == 0 && p.ya_stride % 8 == 0 &&
                   p.yb_stride % 8 == 0 && aligned(p.out, 16) && aligned(p.x, 16) &&
                   aligned(p.ya, 16) && aligned(p.yb, 16) && aligned(p.post_w, 16) &&
                   aligned(p.next_w, 16);
#define AKAP_LNS(TO)                                                                         \
  do {                                                                                       \
    if (!vec) layer_norm_step_kernel<TO><<<p.rows, 256, (size_t)p.d * sizeof(float), s>>>(p); \
    else if (p.d <= 2048) layer_norm_step_vec_kernel<TO, 1><<<p.rows, 256, 0, s>>>(p);       \
    else if (p.d <= 4096) layer_norm_step_vec_kernel<TO, 2><<<p.rows, 256, 0, s>>>(p);       \
    else layer_norm_step_vec_kernel<TO, 4><<<p.rows, 256, 0, s>>>(p);                        \
  } while (0)
  if (out_f32) AKAP_LNS(float);
  else AKAP_LNS(bf16);
#undef AKAP_LNS
}

void launch_clamped_glu(const ClampedGluParams& p, bool f32, hipStream_t s) {
  const int n = p.E * p.F + p.Fs;
  if (p.rows <= 0 || n <= 0) return;
  const bool vec = p.F % 8 == 0 && p.Fs % 8 == 0 && p.gu_stride % 8 == 0 && p.out_stride % 8 == 0 &&
                   aligned(p.gu, 16) && aligned(p.out, 16);
  const int per = vec ? 2048 : 256;
  const dim3 grid(p.rows, (n + per - 1) / per);
  if (f32) {
    if (vec) clamped_glu_kernel<float, 8><<<grid, 256, 0, s>>>(p);
    else clamped_glu_kernel<float, 1><<<grid, 256, 0, s>>>(p);
  } else {
    if (vec) clamped_glu_kernel<bf16, 8><<<grid, 256, 0, s>>>(p);
    else clamped_glu_kernel<bf16, 1><<<grid, 256, 0, s>>>(p);
  }
}

template <typename T>
static void diff_rows(const DiffAttnParams& p, hipStream_t s) {
  const dim3 grid(p.T, (p.H + 3) / 4);
  const size_t sm = (size_t)4 * (2 * p.D + 128) * sizeof(float);
  if (p.Dv <= 64) diff_attention_kernel<T, 1><<<grid, 256, sm, s>>>(p);
  else if (p.Dv <= 128) diff_attention_kernel<T, 2><<<grid, 256, sm, s>>>(p);
  else if (p.Dv <= 256) diff_attention_kernel<T, 4><<<grid, 256, sm, s>>>(p);
  else diff_attention_kernel<T, 8><<<grid, 256, sm, s>>>(p);
}

void launch_diff_attention(const DiffAttnParams& p, bool f32, hipStream_t s) {
  if (p.T <= 0 || p.H <= 0) return;
  if (f32) diff_rows<float>(p, s);
  else diff_rows<bf16>(p, s);
}

}  // namespace akap_stream
