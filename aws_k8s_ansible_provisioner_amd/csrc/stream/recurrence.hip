// Recurrences over a matrix state S [D, V] per head and live sequence: linear attention with a
// fixed decay per head, matrix memory with exponential gates (mLSTM), and the gated delta rule;
// and the head norm + output gate that follows them.
//
// Gates, decays, step sizes, unit norms, the running maximum and the whole state are fp32
// whatever the storage type; every size is a run-time argument.
#include "../kernels/common.h"
#include "stream.h"

namespace akap_stream {

using akap::bf16;
using akap::block_sum;

namespace {

template <typename T>
__device__ __forceinline__ float ldf(const T* p) { return (float)*p; }
template <typename T>
__device__ __forceinline__ void stf(T* p, float v) { *p = (T)v; }

__device__ __forceinline__ void ld4(const float* p, float (&v)[4]) {
  const float4 a = *(const float4*)p;
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
}
__device__ __forceinline__ void ld4(const bf16* p, float (&v)[4]) {
  const akap::bf16x4 a = *(const akap::bf16x4*)p;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = (float)a[i];
}

__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + __expf(-z)); }
__device__ __forceinline__ float gatef(float z, int silu) { return silu ? z * sigmoidf(z) : sigmoidf(z); }
__device__ __forceinline__ float softplusf(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// sum over the DP neighbouring lanes of a group (a power of two; every lane of the wave takes
// part): lane swaps inside a row of 16 on DPP, wider ones by exchange
__device__ __forceinline__ float group_sum(float v, int DP) {
  if (DP > 1) v += akap::dpp_mov<0xB1>(v);
  if (DP > 2) v += akap::dpp_mov<0x4E>(v);
  if (DP > 4) v += akap::dpp_mov<0x141>(v);
  if (DP > 8) v += akap::dpp_mov<0x140>(v);
  if (DP > 16) v += __shfl_xor(v, 16, 64);
  if (DP > 32) v += __shfl_xor(v, 32, 64);
  return v;
}

// ------------------------------------------------------------------ scan
// One workgroup per (sequence, head, VB state columns), at most 256 threads.  A thread keeps
// VR = 4 neighbouring state columns and, of their D rows, 4 groups of four (group j of lane part
// `part` covers d = 4 (j DP + part) ..+4, so the DP lanes of a column group read and write
// consecutive 16-byte pieces of the stored state and of the staged rows).  Rows are staged TC at
// a time; the recurrence then runs over them without a barrier: the DP lanes of a column group
// add their partial sums by lane exchange.  The normaliser of the matrix memory is one more
// column that every column group carries along (its D entries are spread over the same lanes).
// For the delta rule q and k stay as staged: the reciprocals of their lengths, which are scalars
// per token, multiply the sums and the update.
constexpr int kVR = 4;
constexpr int kDreg = 16;
constexpr int kTokens = 16;

// VEC: D a multiple of 4 (16-byte pieces of the stored state; lanes past D or the columns load a
// valid piece that is masked once the first rows are staged, so that the loads of state and rows
// are in flight together)
template <typename T, int MODE, bool VEC>
__global__ __launch_bounds__(256) void recurrence_kernel(RecurrenceParams p) {
  extern __shared__ __align__(16) float lds[];
  constexpr int NJ = kDreg / 4;
  const int DP = p.DP, DPD = DP * kDreg, TC = p.TC, VP = (p.VB + 3) & ~3;
  float* qs = lds;                        // [TC][DPD]
  float* ks = qs + TC * DPD;              // [TC][DPD]
  float* vs = ks + TC * DPD;              // [TC][VP]
  float* os = vs + TC * VP;               // [TC][VP]
  float* g0 = os + TC * VP;               // [TC] decay of the state
  float* g1 = g0 + TC;                    // [TC] input scale | beta
  float* g2 = g1 + TC;                    // [TC] e^-m | 1 / |q|
  float* g3 = g2 + TC;                    // [TC] 1 / |k|
  float* mrun = g3 + TC;                  // [4] running maximum
  const int b = blockIdx.x, h = blockIdx.y, c_lo = blockIdx.z * p.VB;
  const int nv = min(p.VB, p.V - c_lo);   // columns of this workgroup
  const int r0 = p.q_start ? p.q_start[b] : b;
  const int r1 = p.q_start ? p.q_start[b + 1] : b + 1;
  if (r1 <= r0) return;
  const int slot = p.seq_slot[r0];
  if (slot < 0 || slot >= p.num_slots) return;
  const int tid = threadIdx.x, nt = blockDim.x;
  const int hq = h / (p.H / p.G);
  const int v0 = (tid / DP) * kVR, part = tid % DP;
  const bool fresh = p.positions[r0] == 0;
  float* sbase = p.state + (((size_t)slot * p.H + h) * p.V + c_lo) * p.D;
  float* nbase = MODE == kMatrixMemory ? p.n_state + ((size_t)slot * p.H + h) * p.D : nullptr;
  auto load4 = [&](const float* col, int d, bool live) {
    float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
    if (VEC) {
      t = *(const float4*)(col + min(d, p.D - 4));
    } else if (live) {
      if (d < p.D) t.x = col[d];
      if (d + 1 < p.D) t.y = col[d + 1];
      if (d + 2 < p.D) t.z = col[d + 2];
      if (d + 3 < p.D) t.w = col[d + 3];
    }
    return t;
  };
  auto store4 = [&](float* col, int d, float x, float y, float z, float w) {
    if (VEC) {
      if (d < p.D) *(float4*)(col + d) = make_float4(x, y, z, w);
    } else {
      if (d < p.D) col[d] = x;
      if (d + 1 < p.D) col[d + 1] = y;
      if (d + 2 < p.D) col[d + 2] = z;
      if (d + 3 < p.D) col[d + 3] = w;
    }
  };
  float S[kVR][kDreg], N[kDreg];
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int d = 4 * (j * DP + part);
#pragma unroll
    for (int r = 0; r < kVR; ++r) {
      const float4 t = load4(sbase + (size_t)min(v0 + r, nv - 1) * p.D, d, !fresh && v0 + r < nv);
      S[r][4 * j] = t.x; S[r][4 * j + 1] = t.y; S[r][4 * j + 2] = t.z; S[r][4 * j + 3] = t.w;
    }
    float4 t = make_float4(0.f, 0.f, 0.f, 0.f);
    if (MODE == kMatrixMemory) t = load4(nbase, d, !fresh);
    N[4 * j] = t.x; N[4 * j + 1] = t.y; N[4 * j + 2] = t.z; N[4 * j + 3] = t.w;
  }
  if (MODE == kMatrixMemory && tid == 0)
    mrun[0] = fresh ? 0.f : p.m_state[(size_t)slot * p.H + h];
  const float pa = p.pa[h], pb = MODE == kDecay ? 0.f : p.pb[h];
  const float ea = MODE == kDelta ? expf(pa) : 0.f;
  // 16-byte staging: every slice starts and every row strides at a multiple of 4 elements
  const bool vstage = ((p.D | p.V | c_lo | p.qkv_stride | p.q_off | p.k_off | p.v_off) & 3) == 0 &&
                      ((uintptr_t)p.qkv & 15) == 0;
  const float qsc = MODE == kDelta ? 1.0f : p.q_scale;   // the delta rule scales with 1 / |q|
  const bool act = p.act != 0;
  auto on = [&](float z) { return act ? z * sigmoidf(z) : z; };
  int LPT = 64;                           // lanes per token of the per-token phases
  while (LPT * TC > nt && LPT > 1) LPT >>= 1;
  for (int c0 = r0; c0 < r1; c0 += TC) {
    const int n = min(TC, r1 - c0);
    if (vstage) {
      const int Q4 = DPD >> 2;
      for (int e = tid; e < n * Q4; e += nt) {
        const int tk = e / Q4, d = (e - tk * Q4) << 2;
        const T* row = (const T*)p.qkv + (size_t)(c0 + tk) * p.qkv_stride;
        float q4[4] = {0.f, 0.f, 0.f, 0.f}, k4[4] = {0.f, 0.f, 0.f, 0.f};
        if (d < p.D) {
          ld4(row + p.q_off + hq * p.D + d, q4);
          ld4(row + p.k_off + hq * p.D + d, k4);
        }
        *(float4*)(qs + tk * DPD + d) =
            make_float4(on(q4[0]) * qsc, on(q4[1]) * qsc, on(q4[2]) * qsc, on(q4[3]) * qsc);
        *(float4*)(ks + tk * DPD + d) = make_float4(on(k4[0]), on(k4[1]), on(k4[2]), on(k4[3]));
      }
      const int V4 = VP >> 2;
      for (int e = tid; e < n * V4; e += nt) {
        const int tk = e / V4, c = (e - tk * V4) << 2;
        float v4[4] = {0.f, 0.f, 0.f, 0.f};
        if (c < nv)
          ld4((const T*)p.qkv + (size_t)(c0 + tk) * p.qkv_stride + p.v_off + h * p.V + c_lo + c, v4);
        *(float4*)(vs + tk * VP + c) = make_float4(on(v4[0]), on(v4[1]), on(v4[2]), on(v4[3]));
      }
    } else {
      for (int e = tid; e < n * DPD; e += nt) {
        const int tk = e / DPD, d = e % DPD;
        const T* row = (const T*)p.qkv + (size_t)(c0 + tk) * p.qkv_stride;
        qs[e] = d < p.D ? on(ldf(row + p.q_off + hq * p.D + d)) * qsc : 0.f;
        ks[e] = d < p.D ? on(ldf(row + p.k_off + hq * p.D + d)) : 0.f;
      }
      for (int e = tid; e < n * VP; e += nt) {
        const int tk = e / VP, c = e % VP;
        vs[e] = c < nv ? on(ldf((const T*)p.qkv + (size_t)(c0 + tk) * p.qkv_stride + p.v_off +
                                h * p.V + c_lo + c))
                       : 0.f;
      }
    }
    if (tid < n) {
      const T* row = (const T*)p.proj + (size_t)(c0 + tid) * p.proj_stride;
      if (MODE == kDecay) {
        g0[tid] = pa;
      } else if (MODE == kMatrixMemory) {
        const float f = p.cap * tanhf((ldf(row + p.a_off + h) + pa) / p.cap);
        g0[tid] = -softplusf(-f);
        g1[tid] = p.cap * tanhf((ldf(row + p.b_off + h) + pb) / p.cap);
      } else {
        g0[tid] = expf(-ea * softplusf(ldf(row + p.a_off + h) + pb));
        g1[tid] = 1.0f / (1.0f + expf(-ldf(row + p.b_off + h)));
      }
    }
    __syncthreads();
    if (MODE == kMatrixMemory) {
      if (tid == 0) {
        float m = mrun[0];
        for (int tk = 0; tk < n; ++tk) {
          const float f = g0[tk], i = g1[tk], m2 = fmaxf(f + m, i);
          g0[tk] = expf(f + m - m2);
          g1[tk] = expf(i - m2);
          g2[tk] = expf(-m2);
          m = m2;
        }
        mrun[0] = m;
      }
      __syncthreads();
    } else if (MODE == kDelta) {
      for (int tk = tid / LPT; tk < n; tk += nt / LPT) {
        const int ln = tid % LPT;
        float sq = 0.f, sk = 0.f;
        for (int d = ln; d < p.D; d += LPT) {
          const float a = qs[tk * DPD + d], c = ks[tk * DPD + d];
          sq += a * a;
          sk += c * c;
        }
        for (int o = LPT >> 1; o > 0; o >>= 1) {
          sq += __shfl_xor(sq, o, 64);
          sk += __shfl_xor(sk, o, 64);
        }
        if (ln == 0) {
          g2[tk] = p.q_scale / sqrtf(sq + 1e-6f);
          g3[tk] = 1.0f / sqrtf(sk + 1e-6f);
        }
      }
      __syncthreads();
    }
    if (VEC && c0 == r0) {
#pragma unroll
      for (int i = 0; i < kDreg; ++i) {
        const bool in = !fresh && 4 * ((i >> 2) * DP + part) < p.D;
#pragma unroll
        for (int r = 0; r < kVR; ++r) S[r][i] = in && v0 + r < nv ? S[r][i] : 0.f;
        if (MODE == kMatrixMemory) N[i] = in ? N[i] : 0.f;
      }
    }
    // the recurrence
    for (int tk = 0; tk < n; ++tk) {
      float4 vv = make_float4(0.f, 0.f, 0.f, 0.f);
      if (v0 < VP) vv = *(const float4*)(vs + tk * VP + v0);
      float vr[kVR] = {vv.x, vv.y, vv.z, vv.w};
      const float* kq = ks + tk * DPD + 4 * part;
      const float* qq = qs + tk * DPD + 4 * part;
      const float dec = g0[tk];
      float acc[kVR] = {0.f, 0.f, 0.f, 0.f};
      float accn = 0.f;
      if (MODE == kDelta) {
        float kk[kDreg];
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
          const float4 k4 = *(const float4*)(kq + 4 * j * DP);
          kk[4 * j] = k4.x; kk[4 * j + 1] = k4.y; kk[4 * j + 2] = k4.z; kk[4 * j + 3] = k4.w;
        }
        float seen[kVR] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < kDreg; ++i)
#pragma unroll
          for (int r = 0; r < kVR; ++r) {
            S[r][i] *= dec;
            seen[r] = fmaf(S[r][i], kk[i], seen[r]);
          }
#pragma unroll
        for (int r = 0; r < kVR; ++r) seen[r] = group_sum(seen[r], DP);
        const float beta = g1[tk], ik = g3[tk];
#pragma unroll
        for (int r = 0; r < kVR; ++r) vr[r] = beta * (vr[r] - ik * seen[r]) * ik;
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
          const float4 q4 = *(const float4*)(qq + 4 * j * DP);
          const float qv[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
          for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int r = 0; r < kVR; ++r) {
              S[r][4 * j + i] = fmaf(kk[4 * j + i], vr[r], S[r][4 * j + i]);
              acc[r] = fmaf(S[r][4 * j + i], qv[i], acc[r]);
            }
        }
      } else {
        if (MODE == kMatrixMemory) {
          const float add = g1[tk];
#pragma unroll
          for (int r = 0; r < kVR; ++r) vr[r] *= add;
        }
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
          const float4 k4 = *(const float4*)(kq + 4 * j * DP);
          const float4 q4 = *(const float4*)(qq + 4 * j * DP);
          const float kv[4] = {k4.x, k4.y, k4.z, k4.w}, qv[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
          for (int i = 0; i < 4; ++i) {
#pragma unroll
            for (int r = 0; r < kVR; ++r) {
              S[r][4 * j + i] = fmaf(dec, S[r][4 * j + i], kv[i] * vr[r]);
              acc[r] = fmaf(S[r][4 * j + i], qv[i], acc[r]);
            }
            if (MODE == kMatrixMemory) {
              N[4 * j + i] = fmaf(dec, N[4 * j + i], kv[i] * g1[tk]);
              accn = fmaf(N[4 * j + i], qv[i], accn);
            }
          }
        }
      }
#pragma unroll
      for (int r = 0; r < kVR; ++r) acc[r] = group_sum(acc[r], DP);
      if (MODE == kMatrixMemory) accn = group_sum(accn, DP);
      float f = 1.0f;
      if (MODE == kMatrixMemory) f = 1.0f / (fmaxf(fabsf(accn), g2[tk]) + 1e-6f);
      if (MODE == kDelta) f = g2[tk];
      if (v0 < VP && part == 0)
        *(float4*)(os + tk * VP + v0) = make_float4(acc[0] * f, acc[1] * f, acc[2] * f, acc[3] * f);
    }
    __syncthreads();
    if (p.raw) {
      for (int e = tid; e < n * nv; e += nt) {
        const int tk = e / nv, c = e - tk * nv;
        p.raw[((size_t)(c0 + tk) * p.H + h) * p.V + c_lo + c] = os[tk * VP + c];
      }
    } else {
      // the head norm over its V entries, the weights and the output gate: LPT lanes per token
      for (int tk = tid / LPT; tk < n; tk += nt / LPT) {
        const int ln = tid % LPT;
        float ss = 0.f;
        for (int c = ln; c < p.V; c += LPT) {
          const float f = os[tk * VP + c];
          ss += f * f;
        }
        for (int o = LPT >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
        const float inv = 1.0f / sqrtf(ss / (float)p.V + p.eps);
        const T* g = (const T*)p.proj + (size_t)(c0 + tk) * p.proj_stride + p.g_off + h * p.V;
        T* o = (T*)p.out + (size_t)(c0 + tk) * p.out_stride + h * p.V;
        for (int c = ln; c < p.V; c += LPT)
          stf(o + c, os[tk * VP + c] * inv * p.norm_w[h * p.V + c] * gatef(ldf(g + c), p.gate_act));
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int d = 4 * (j * DP + part);
#pragma unroll
    for (int r = 0; r < kVR; ++r)
      if (v0 + r < nv)
        store4(sbase + (size_t)(v0 + r) * p.D, d, S[r][4 * j], S[r][4 * j + 1],
               S[r][4 * j + 2], S[r][4 * j + 3]);
    if (MODE == kMatrixMemory && v0 == 0 && blockIdx.z == 0)
      store4(nbase, d, N[4 * j], N[4 * j + 1], N[4 * j + 2], N[4 * j + 3]);
  }
  if (MODE == kMatrixMemory && tid == 0 && blockIdx.z == 0)
    p.m_state[(size_t)slot * p.H + h] = mrun[0];
}

// ------------------------------------------------------------------ one token per sequence
// The same for steps of single rows, which only stream the state in and out: a workgroup per
// (row, head), up to 1024 threads.  Nothing is staged: a lane loads the pieces of q and k that
// meet its state rows, everything before the head norm happens inside the lanes of a column
// group, and all loads are issued together.  Sizes in fours, aligned.
template <typename T, int MODE, int DREG>
__global__ __launch_bounds__(1024) void recurrence_step_kernel(RecurrenceParams p) {
  __shared__ float scratch[16];
  constexpr int NJ = DREG / 4;
  const int DP = p.DP;
  const int t = blockIdx.x, h = blockIdx.y;
  const int slot = p.seq_slot[t];
  if (slot < 0 || slot >= p.num_slots) return;
  const int tid = threadIdx.x, hq = h / (p.H / p.G);
  const int v0 = (tid / DP) * kVR, part = tid % DP;
  const bool col = v0 < p.V;
  const int vc = col ? v0 : p.V - kVR;
  const T* row = (const T*)p.qkv + (size_t)t * p.qkv_stride;
  const T* pr = (const T*)p.proj + (size_t)t * p.proj_stride;
  float* sp = p.state + (((size_t)slot * p.H + h) * p.V + vc) * p.D;
  float* np = MODE == kMatrixMemory ? p.n_state + ((size_t)slot * p.H + h) * p.D : nullptr;
  float q[DREG], k[DREG], v[kVR];
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int d = min(4 * (j * DP + part), p.D - 4);
    float q4[4], k4[4];
    ld4(row + p.q_off + hq * p.D + d, q4);
    ld4(row + p.k_off + hq * p.D + d, k4);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      q[4 * j + i] = q4[i];
      k[4 * j + i] = k4[i];
    }
  }
  ld4(row + p.v_off + h * p.V + vc, v);
  akap::f32x4 S[kVR][NJ], N[NJ];
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int d = min(4 * (j * DP + part), p.D - 4);
#pragma unroll
    for (int r = 0; r < kVR; ++r) S[r][j] = *(const akap::f32x4*)(sp + r * p.D + d);
    if (MODE == kMatrixMemory) N[j] = *(const akap::f32x4*)(np + d);
  }
  const bool fresh = p.positions[t] == 0;
  float dec, add = 1.f, floor_m = 0.f, m2 = 0.f;
  if (MODE == kDecay) {
    dec = p.pa[h];
  } else if (MODE == kMatrixMemory) {
    const float f = -softplusf(-p.cap * tanhf((ldf(pr + p.a_off + h) + p.pa[h]) / p.cap));
    const float i = p.cap * tanhf((ldf(pr + p.b_off + h) + p.pb[h]) / p.cap);
    const float m = fresh ? 0.f : p.m_state[(size_t)slot * p.H + h];
    m2 = fmaxf(f + m, i);
    dec = expf(f + m - m2);
    add = expf(i - m2);
    floor_m = expf(-m2);
  } else {
    dec = expf(-expf(p.pa[h]) * softplusf(ldf(pr + p.a_off + h) + p.pb[h]));
    add = 1.0f / (1.0f + expf(-ldf(pr + p.b_off + h)));   // the step size
  }
  if (fresh) dec = 0.f;
  const float qs = MODE == kDelta ? 1.0f : p.q_scale;
#pragma unroll
  for (int i = 0; i < DREG; ++i) {
    const bool in = 4 * ((i >> 2) * DP + part) < p.D;
    if (p.act) {
      q[i] *= sigmoidf(q[i]);
      k[i] *= sigmoidf(k[i]);
    }
    q[i] = in ? q[i] * qs : 0.f;
    k[i] = in ? k[i] : 0.f;
  }
  if (p.act) {
#pragma unroll
    for (int r = 0; r < kVR; ++r) v[r] *= sigmoidf(v[r]);
  }
  // a fresh row: the slot's stale contents (which may be anything) do not enter
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
      for (int r = 0; r < kVR; ++r) S[r][j][i] = fresh ? 0.f : S[r][j][i];
      if (MODE == kMatrixMemory) N[j][i] = fresh ? 0.f : N[j][i];
    }
  }
  float acc[kVR] = {0.f, 0.f, 0.f, 0.f}, f = 1.0f;
  if (MODE == kDelta) {
    float seen[kVR] = {0.f, 0.f, 0.f, 0.f}, sq = 0.f, sk = 0.f;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
#pragma unroll
      for (int r = 0; r < kVR; ++r) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          S[r][j][i] *= dec;
          seen[r] = fmaf(S[r][j][i], k[4 * j + i], seen[r]);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        sq = fmaf(q[4 * j + i], q[4 * j + i], sq);
        sk = fmaf(k[4 * j + i], k[4 * j + i], sk);
      }
    }
#pragma unroll
    for (int r = 0; r < kVR; ++r) seen[r] = group_sum(seen[r], DP);
    const float ik = 1.0f / sqrtf(group_sum(sk, DP) + 1e-6f);
    f = p.q_scale / sqrtf(group_sum(sq, DP) + 1e-6f);
#pragma unroll
    for (int r = 0; r < kVR; ++r) v[r] = add * (v[r] - ik * seen[r]) * ik;
    dec = 1.f;
  } else {
#pragma unroll
    for (int r = 0; r < kVR; ++r) v[r] *= add;
  }
  float accn = 0.f;
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
      for (int r = 0; r < kVR; ++r) {
        S[r][j][i] = fmaf(dec, S[r][j][i], k[4 * j + i] * v[r]);
        acc[r] = fmaf(S[r][j][i], q[4 * j + i], acc[r]);
      }
      if (MODE == kMatrixMemory) {
        N[j][i] = fmaf(dec, N[j][i], k[4 * j + i] * add);
        accn = fmaf(N[j][i], q[4 * j + i], accn);
      }
    }
  }
  // the state leaves before the sums are finished (the normaliser: every column group has read it
  // by the barrier below)
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int d = 4 * (j * DP + part);
    if (col && d < p.D)
#pragma unroll
      for (int r = 0; r < kVR; ++r) *(akap::f32x4*)(sp + r * p.D + d) = S[r][j];
  }
#pragma unroll
  for (int r = 0; r < kVR; ++r) acc[r] = group_sum(acc[r], DP);
  if (MODE == kMatrixMemory) f = 1.0f / (fmaxf(fabsf(group_sum(accn, DP)), floor_m) + 1e-6f);
  float ss = 0.f;
#pragma unroll
  for (int r = 0; r < kVR; ++r) {
    acc[r] = col ? acc[r] * f : 0.f;
    ss += acc[r] * acc[r];
  }
  ss = block_sum(part == 0 ? ss : 0.f, scratch);
  if (MODE == kMatrixMemory && v0 == 0) {
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int d = 4 * (j * DP + part);
      if (d < p.D) *(akap::f32x4*)(np + d) = N[j];
    }
    if (part == 0) p.m_state[(size_t)slot * p.H + h] = m2;
  }
  if (!col || part != 0) return;
  if (p.raw) {
    *(float4*)(p.raw + ((size_t)t * p.H + h) * p.V + v0) = make_float4(acc[0], acc[1], acc[2], acc[3]);
    return;
  }
  const float inv = 1.0f / sqrtf(ss / (float)p.V + p.eps);
  const T* g = pr + p.g_off + h * p.V + v0;
  T* o = (T*)p.out + (size_t)t * p.out_stride + h * p.V + v0;
#pragma unroll
  for (int r = 0; r < kVR; ++r)
    stf(o + r, acc[r] * inv * p.norm_w[h * p.V + v0 + r] * gatef(ldf(g + r), p.gate_act));
}

// ------------------------------------------------------------------ head norm + output gate
// one workgroup of four waves per row: a part per wave when there are several, else all threads
template <typename T>
__global__ __launch_bounds__(256) void norm_gate_kernel(T* __restrict__ out, int out_stride,
                                                        const float* __restrict__ y,
                                                        const T* __restrict__ gate, int gate_stride,
                                                        const float* __restrict__ w,
                                                        const float* __restrict__ den,
                                                        const float* __restrict__ floor, int silu,
                                                        int n, int groups, float eps, int vec) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, part = n / groups;
  const float* yr = y + (size_t)t * n;
  const T* gr = gate + (size_t)t * gate_stride;
  T* o = out + (size_t)t * out_stride;
  const int wave = threadIdx.x >> 6;
  const bool shared = groups == 1;
  const int step = shared ? 256 : 64, ln = shared ? threadIdx.x : (threadIdx.x & 63);
  for (int g = shared ? 0 : wave; g < groups; g += shared ? 1 : 4) {
    const int c0 = g * part;
    float scale = 1.0f;
    if (den) {
      const size_t i = (size_t)t * groups + g;
      scale = 1.0f / (fmaxf(fabsf(den[i]), floor[i]) + 1e-6f);
    }
    float ss = 0.f;
    if (vec) {
      for (int c = ln * 4; c < part; c += step * 4) {
        const float4 v = *(const float4*)(yr + c0 + c);
        ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
      }
    } else {
      for (int c = ln; c < part; c += step) ss += yr[c0 + c] * yr[c0 + c];
    }
    ss = shared ? block_sum(ss, scratch) : akap::wave_sum(ss);
    // eps inside the root of the divided values
    const float inv = scale / sqrtf(ss * scale * scale / (float)part + eps);
    if (vec) {
      for (int c = ln * 4; c < part; c += step * 4) {
        const float4 v = *(const float4*)(yr + c0 + c);
        const float4 wv = *(const float4*)(w + c0 + c);
        float gv[4];
        ld4(gr + c0 + c, gv);
        T r[4] = {(T)(v.x * inv * wv.x * gatef(gv[0], silu)), (T)(v.y * inv * wv.y * gatef(gv[1], silu)),
                  (T)(v.z * inv * wv.z * gatef(gv[2], silu)), (T)(v.w * inv * wv.w * gatef(gv[3], silu))};
        __builtin_memcpy(o + c0 + c, r, sizeof(r));
      }
    } else {
      for (int c = ln; c < part; c += step)
        stf(o + c0 + c, yr[c0 + c] * inv * w[c0 + c] * gatef(ldf(gr + c0 + c), silu));
    }
  }
}

// the same with the row's values, gates and weights held in registers (sizes in fours, aligned):
// LG lanes per part (a power of two up to a wave, or all 256 threads for one part), NV groups of
// four per lane
template <typename T, int NV, bool ALL>
__global__ __launch_bounds__(256) void norm_gate_vec_kernel(
    T* __restrict__ out, int out_stride, const float* __restrict__ y, const T* __restrict__ gate,
    int gate_stride, const float* __restrict__ w, const float* __restrict__ den,
    const float* __restrict__ floor, int silu, int n, int groups, int LG, float eps) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, part = n / groups;
  const float* yr = y + (size_t)t * n;
  const T* gr = gate + (size_t)t * gate_stride;
  T* o = out + (size_t)t * out_stride;
  const int lanes = ALL ? 256 : LG, ln = ALL ? threadIdx.x : threadIdx.x & (LG - 1);
  for (int g = ALL ? 0 : threadIdx.x / LG; g < groups; g += ALL ? 1 : 256 / LG) {
    const int c0 = g * part;
    float4 v[NV], wv[NV];
    float gv[NV][4];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * lanes + ln) * 4;
      if (c < part) {
        v[k] = *(const float4*)(yr + c0 + c);
        ld4(gr + c0 + c, gv[k]);
        wv[k] = *(const float4*)(w + c0 + c);
      } else {
        v[k] = wv[k] = make_float4(0.f, 0.f, 0.f, 0.f);
      }
    }
#pragma unroll
    for (int k = 0; k < NV; ++k)
      ss += v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w;
    float scale = 1.0f;
    if (den) {
      const size_t i = (size_t)t * groups + g;
      scale = 1.0f / (fmaxf(fabsf(den[i]), floor[i]) + 1e-6f);
    }
    if (ALL) {
      ss = block_sum(ss, scratch);
    } else {
      for (int x = LG >> 1; x > 0; x >>= 1) ss += __shfl_xor(ss, x, 64);
    }
    const float inv = scale / sqrtf(ss * scale * scale / (float)part + eps);
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = (k * lanes + ln) * 4;
      if (c >= part) continue;
      T r[4] = {(T)(v[k].x * inv * wv[k].x * gatef(gv[k][0], silu)),
                (T)(v[k].y * inv * wv[k].y * gatef(gv[k][1], silu)),
                (T)(v[k].z * inv * wv[k].z * gatef(gv[k][2], silu)),
                (T)(v[k].w * inv * wv[k].w * gatef(gv[k][3], silu))};
      __builtin_memcpy(o + c0 + c, r, sizeof(r));
    }
  }
}

// lanes per column group and columns per workgroup of the scan
void scan_shape(int D, int V, int* dp, int* vb) {
  int p = 1;
  while (p * kDreg < D) p <<= 1;
  *dp = p;
  const int cols = kVR * (256 / p);
  *vb = V <= cols ? V : cols;
}

// state rows per thread of the single-row form (0: too large for a workgroup) and its lanes per
// column group
int step_shape(int D, int V, int* dp) {
  for (int dreg : {8, 16}) {
    int p = 1;
    while (p * dreg < D) p <<= 1;
    *dp = p;
    if (p <= 64 && (V / kVR) * p <= 1024) return dreg;
  }
  return 0;
}

}  // namespace

// ================================================================== launchers
bool recurrence_supported(int D, int V) { return D >= 1 && D <= 64 * 16 && V >= 1; }

bool recurrence_fused(int D, int V) {
  int dp, vb;
  scan_shape(D, V, &dp, &vb);
  return vb == V;
}

bool recurrence_step_supported(int D, int V) {
  int dp;
  return D >= 4 && V >= 4 && D % 4 == 0 && V % 4 == 0 && step_shape(D, V, &dp) > 0;
}

void launch_recurrence_step(RecurrenceParams p, int mode, bool f32, hipStream_t s) {
  if (p.num_seqs <= 0) return;
  const int dreg = step_shape(p.D, p.V, &p.DP);
  const int nt = ((p.V / kVR * p.DP + 63) / 64) * 64;
  const dim3 grid(p.num_seqs, p.H);
#define AKAP_ST1(TY, R)                                                                       \
  do {                                                                                        \
    if (mode == kDecay) recurrence_step_kernel<TY, kDecay, R><<<grid, nt, 0, s>>>(p);         \
    else if (mode == kMatrixMemory)                                                           \
      recurrence_step_kernel<TY, kMatrixMemory, R><<<grid, nt, 0, s>>>(p);                    \
    else recurrence_step_kernel<TY, kDelta, R><<<grid, nt, 0, s>>>(p);                        \
  } while (0)
#define AKAP_ST(TY)                     \
  do {                                  \
    if (dreg == 8) AKAP_ST1(TY, 8);     \
    else AKAP_ST1(TY, 16);              \
  } while (0)
  if (f32) AKAP_ST(float);
  else AKAP_ST(bf16);
#undef AKAP_ST
#undef AKAP_ST1
}

void launch_recurrence(RecurrenceParams p, int mode, bool f32, hipStream_t s) {
  if (p.num_seqs <= 0) return;
  scan_shape(p.D, p.V, &p.DP, &p.VB);
  const int groups = (p.VB + kVR - 1) / kVR;
  const int nt = ((groups * p.DP + 63) / 64) * 64;
  const int vp = (p.VB + 3) & ~3;
  p.TC = p.q_start ? kTokens : 1;
  auto need = [&](int tc) {
    return (size_t)(tc * (2 * p.DP * kDreg + 2 * vp + 4) + 4) * sizeof(float);
  };
  while (p.TC > 1 && need(p.TC) > 65536) p.TC >>= 1;
  const size_t lds = need(p.TC);
  const dim3 grid(p.num_seqs, p.H, (p.V + p.VB - 1) / p.VB);
#define AKAP_REC1(TY, VC)                                                                      \
  do {                                                                                        \
    if (mode == kDecay) recurrence_kernel<TY, kDecay, VC><<<grid, nt, lds, s>>>(p);           \
    else if (mode == kMatrixMemory)                                                           \
      recurrence_kernel<TY, kMatrixMemory, VC><<<grid, nt, lds, s>>>(p);                      \
    else recurrence_kernel<TY, kDelta, VC><<<grid, nt, lds, s>>>(p);                          \
  } while (0)
#define AKAP_REC(TY)                       \
  do {                                     \
    if (p.D % 4 == 0) AKAP_REC1(TY, true); \
    else AKAP_REC1(TY, false);             \
  } while (0)
  if (f32) AKAP_REC(float);
  else AKAP_REC(bf16);
#undef AKAP_REC
#undef AKAP_REC1
}

void launch_norm_gate(void* out, int out_stride, const float* y, const void* gate, int gate_stride,
                      const float* w, const float* den, const float* floor, bool f32, int act,
                      int rows, int n, int groups, float eps, hipStream_t s) {
  if (rows <= 0) return;
  const int part = n / groups, es = f32 ? 4 : 2;
  auto al = [](const void* p, int bytes) { return ((uintptr_t)p % bytes) == 0; };
  const int vec = part % 4 == 0 && out_stride % 4 == 0 && gate_stride % 4 == 0 && al(y, 16) &&
                  al(w, 16) && al(out, 4 * es) && al(gate, 4 * es);
  int lg = 1;
  while (lg < 64 && lg * 4 < part) lg <<= 1;
  const bool all = groups == 1 && part > 256;
  const int nv = (part + (all ? 1023 : lg * 4 - 1)) / (all ? 1024 : lg * 4);
  if (vec && nv <= 4) {
#define AKAP_NG1(TY, N, A)                                                                        \
  norm_gate_vec_kernel<TY, N, A><<<rows, 256, 0, s>>>((TY*)out, out_stride, y, (const TY*)gate,   \
                                                      gate_stride, w, den, floor, act, n, groups, \
                                                      lg, eps)
#define AKAP_NG(TY)                                                               \
  do {                                                                            \
    if (all) {                                                                    \
      if (nv == 1) AKAP_NG1(TY, 1, true);                                         \
      else if (nv == 2) AKAP_NG1(TY, 2, true);                                    \
      else AKAP_NG1(TY, 4, true);                                                 \
    } else {                                                                      \
      if (nv == 1) AKAP_NG1(TY, 1, false);                                        \
      else if (nv == 2) AKAP_NG1(TY, 2, false);                                   \
      else AKAP_NG1(TY, 4, false);                                                \
    }                                                                             \
  } while (0)
    if (f32) AKAP_NG(float);
    else AKAP_NG(bf16);
#undef AKAP_NG
#undef AKAP_NG1
    return;
  }
  if (f32)
    norm_gate_kernel<float><<<rows, 256, 0, s>>>((float*)out, out_stride, y, (const float*)gate,
                                                 gate_stride, w, den, floor, act, n, groups, eps,
                                                 vec);
  else
    norm_gate_kernel<bf16><<<rows, 256, 0, s>>>((bf16*)out, out_stride, y, (const bf16*)gate,
                                                gate_stride, w, den, floor, act, n, groups, eps,
                                                vec);
}

}  // namespace akap_stream
