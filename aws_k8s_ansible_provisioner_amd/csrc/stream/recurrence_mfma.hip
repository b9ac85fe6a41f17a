// The recurrences of recurrence.hip for prompt chunks on the matrix cores (bf16 storage): a
// sequence's rows are cut into chunks of 64 tokens, a first launch prepares every chunk of every
// head side by side, a second one walks the chunks of a (sequence, head) with the fp32 state in
// accumulator registers.
//
// With L_t the sum of the log decays from the chunk's start through token t, S0 the state before
// the chunk, and c_s / d_t the scalars of a key and a query (input scale or 1 / |k|; q's scale
// or that over |q|):
//   o_t   = d_t e^(L_t) q_t S0 + sum_{s <= t} P_ts x_s,   P_ts = d_t e^(L_t - L_s) c_s (q_t . k_s)
//   S_end = e^(L_end) S0 + sum_s k_s (e^(L_end - L_s) c_s x_s)^T
// with x_s = v_s for the plain recurrences; for the delta rule x = u solves
//   (I + A) u = beta v - beta e^L c (K S0),   A_ts = beta_t e^(L_t - L_s) c_t c_s (k_t . k_s), s < t
// (the unit-vector recurrence with the lengths pulled out of the products), whose unit lower
// triangular inverse depends on the keys and gates alone and is prepared per chunk.
//
// bf16 operands are the stored q, k, v (exact); every fp32 quantity that has to be an operand
// (S0, P, u, the inverse) is split into a bf16 pair hi + lo, so products keep about 16 bits of
// it; sums are fp32.
//
// Operand layouts (v_mfma_f32_16x16x32_bf16, g = lane >> 4): an accumulator lane holds column
// l & 15 and rows 4 g + j in registers j.  Two neighbouring tiles read as the B operand of the
// next product are 8 of the 32 contraction indices of a block, in the order
// slot 8 g + e <-> index 16 (e >> 2) + 4 g + (e & 3).  A operands are stored in that order (a
// fragment = 64 lanes x 8 elements, 1 KB, one 16-byte load per lane), so the state, the solved
// rows and the outputs of one product feed the next without leaving the registers.
#include <type_traits>

#include "../kernels/common.h"
#include "stream.h"

namespace akap_stream {

using akap::bf16;
using akap::bf16x4;
using akap::bf16x8;
using akap::f32x4;

namespace {

constexpr int kC = 64;          // tokens of a chunk
constexpr int kFrag = 512;      // elements of a fragment
constexpr int kPT = 12;         // fragments of P (and of the inverse): 6 of hi, 6 of lo
constexpr int kSc = 4 * kC;     // floats of scalars per (chunk, head)

__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + __expf(-z)); }
__device__ __forceinline__ float softplusf(float z) { return z > 20.f ? z : log1pf(expf(z)); }

__device__ __forceinline__ f32x4 mfma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// fragment of P and of the inverse: tile of 16 rows tt, block of 32 columns kb (kb <= tt / 2)
__device__ __forceinline__ constexpr int tri(int tt, int kb) {
  return tt < 2 ? tt : 2 + (tt - 2) * 2 + kb;
}

// two floats rounded to a pair of bf16
__device__ __forceinline__ uint32_t pack2(float a, float b) {
  const akap::f32x2 f = {a, b};
  return __builtin_bit_cast(uint32_t, __builtin_convertvector(f, akap::bf16x2));
}

__device__ __forceinline__ void split8(const float (&v)[8], bf16x8& hi, bf16x8& lo) {
  uint32_t h[4], l[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    h[i] = pack2(v[2 * i], v[2 * i + 1]);
    l[i] = pack2(v[2 * i] - __uint_as_float(h[i] << 16),
                 v[2 * i + 1] - __uint_as_float(h[i] & 0xffff0000u));
  }
  hi = __builtin_bit_cast(bf16x8, h);
  lo = __builtin_bit_cast(bf16x8, l);
}

// entries of a chunk buffer: sequence b (counted from the first chunked one) owns those from
// (first row - row0) / 64 + b on
__device__ __forceinline__ int chunk_base(const int32_t* q_start, int b, int row0) {
  return (q_start[b] - row0) / kC + b;
}

// ------------------------------------------------------------------ chunk preparation
// One workgroup of four waves per (chunk, head).
template <int MODE, int DT>
__global__ __launch_bounds__(256) void chunk_prep_kernel(ChunkParams p) {
  constexpr int D = DT * 32, LS = D + 8;
  constexpr int AS = 68;
  __shared__ __align__(16) bf16 qs[kC * LS];
  __shared__ __align__(16) bf16 ks[kC * LS];
  __shared__ __align__(16) float am[MODE == kDelta ? kC * AS : 4];
  __shared__ float Ls[kC], ct[kC], cs[kC], bt[kC];
  const RecurrenceParams& r = p.r;
  const int h = blockIdx.y, entry = blockIdx.x;
  int lo = 0, hi = r.num_seqs - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (chunk_base(r.q_start, mid, p.row0) <= entry) lo = mid; else hi = mid - 1;
  }
  const int b = lo;
  const int first = r.q_start[b], end = r.q_start[b + 1];
  const int r0 = first + (entry - chunk_base(r.q_start, b, p.row0)) * kC;
  if (r0 < first || r0 >= end) return;
  const int slot = r.seq_slot[first];
  if (slot < 0 || slot >= r.num_slots) return;
  const int n = min(kC, end - r0);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, g4 = (lane >> 4) * 4, ln = lane & 15;
  const int rep = r.H / r.G, hq = h / rep;
  const size_t ch = (size_t)entry * r.H + h, cg = (size_t)entry * r.G + hq;

  // q and k of the chunk, activated, rows past its end zero
  for (int e = tid; e < kC * (D / 8); e += 256) {
    const int row = e / (D / 8), c = (e - row * (D / 8)) * 8;
    bf16x8 q8, k8;
#pragma unroll
    for (int i = 0; i < 8; ++i) q8[i] = k8[i] = (bf16)0.f;
    if (row < n) {
      const bf16* src = (const bf16*)r.qkv + (size_t)(r0 + row) * r.qkv_stride + hq * D + c;
      q8 = *(const bf16x8*)(src + r.q_off);
      k8 = *(const bf16x8*)(src + r.k_off);
      if (MODE == kDecay && r.act) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const float a = (float)q8[i], c2 = (float)k8[i];
          q8[i] = (bf16)(a * sigmoidf(a));
          k8[i] = (bf16)(c2 * sigmoidf(c2));
        }
      }
    }
    *(bf16x8*)(qs + row * LS + c) = q8;
    *(bf16x8*)(ks + row * LS + c) = k8;
  }
  __syncthreads();
  if (MODE == kDelta) {
    // lengths: four lanes per token
    const int row = tid >> 2;
    float sq = 0.f, sk = 0.f;
    for (int c = (tid & 3) * 8; c < D; c += 32) {
      const bf16x8 q8 = *(const bf16x8*)(qs + row * LS + c), k8 = *(const bf16x8*)(ks + row * LS + c);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        sq += (float)q8[i] * (float)q8[i];
        sk += (float)k8[i] * (float)k8[i];
      }
    }
    sq += __shfl_xor(sq, 1, 64);
    sk += __shfl_xor(sk, 1, 64);
    sq += __shfl_xor(sq, 2, 64);
    sk += __shfl_xor(sk, 2, 64);
    if ((tid & 3) == 0) {
      ct[row] = r.q_scale / sqrtf(sq + 1e-6f);
      cs[row] = 1.0f / sqrtf(sk + 1e-6f);
    }
    __syncthreads();
  }
  if (wave == 0) {
    const int row = r0 + min(lane, n - 1);
    const bool live = lane < n;
    float la = 0.f, beta = 0.f, c_s = 1.f, d_t = r.q_scale;
    if (MODE == kDecay) {
      la = fmaxf(logf(r.pa[h]), -1e4f);
    } else if (MODE == kMatrixMemory) {
      la = p.la[(size_t)row * r.H + h];
      c_s = p.lb[(size_t)row * r.H + h];
    } else {
      const bf16* pr = (const bf16*)r.proj + (size_t)row * r.proj_stride;
      la = -expf(r.pa[h]) * softplusf((float)pr[r.a_off + h] + r.pb[h]);
      beta = 1.0f / (1.0f + expf(-(float)pr[r.b_off + h]));
      c_s = cs[lane];
      d_t = ct[lane];
    }
    if (!live) { la = 0.f; beta = 0.f; c_s = 0.f; }
    float L = la;
    for (int o = 1; o < 64; o <<= 1) {
      const float t = __shfl_up(L, o, 64);
      if (lane >= o) L += t;
    }
    const float Lend = __shfl(L, 63, 64), eL = expf(L);
    Ls[lane] = L;
    ct[lane] = d_t;
    cs[lane] = c_s;
    bt[lane] = beta;
    float* sc = p.sc + ch * kSc;
    sc[lane] = eL * d_t;
    sc[kC + lane] = expf(Lend - L) * c_s;
    sc[2 * kC + lane] = beta;
    sc[3 * kC + lane] = beta * eL * c_s;
    if (lane == 0) p.eend[ch] = expf(Lend);
  }
  __syncthreads();
  // P (and A): the transposed product, key tiles x a query tile, so that a lane holds a query's
  // row; a wave takes the 16 queries of its number
  {
    const int tt = wave, t = tt * 16 + ln;
    const float Lt = Ls[t], dt = ct[t], at = MODE == kDelta ? bt[t] * cs[t] : 0.f;
    bf16* pf = (bf16*)p.pf + ch * kPT * kFrag;
    for (int kb = 0; kb <= tt >> 1; ++kb) {
      float v[8];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const int st = 2 * kb + half;
        f32x4 qk = {0.f, 0.f, 0.f, 0.f}, kk = {0.f, 0.f, 0.f, 0.f};
        if (st <= tt) {
#pragma unroll
          for (int k = 0; k < DT; ++k) {
            const bf16x8 a = *(const bf16x8*)(ks + (st * 16 + ln) * LS + k * 32 + g4 * 2);
            const bf16x8 q = *(const bf16x8*)(qs + t * LS + k * 32 + g4 * 2);
            qk = mfma(a, q, qk);
            if (MODE == kDelta) {
              const bf16x8 k8 = *(const bf16x8*)(ks + t * LS + k * 32 + g4 * 2);
              kk = mfma(a, k8, kk);
            }
          }
        }
        float av[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int s = st * 16 + g4 + e;
          const float w = __expf(fminf(Lt - Ls[s], 0.f)) * cs[s];
          v[half * 4 + e] = s <= t ? qk[e] * w * dt : 0.f;
          av[e] = s < t ? kk[e] * w * at : 0.f;
        }
        if (MODE == kDelta)
          *(float4*)(am + t * AS + st * 16 + g4) = make_float4(av[0], av[1], av[2], av[3]);
      }
      bf16x8 vh, vl;
      split8(v, vh, vl);
      const int idx = tri(tt, kb);
      *(bf16x8*)(pf + idx * kFrag + lane * 8) = vh;
      *(bf16x8*)(pf + (6 + idx) * kFrag + lane * 8) = vl;
    }
  }
  // fragments of q, k (rows = tokens) and of k transposed (rows = dimensions), once per key head
  if (h % rep == 0) {
    bf16* qf = (bf16*)p.qf + cg * 4 * DT * kFrag;
    bf16* kf = (bf16*)p.kf + cg * 4 * DT * kFrag;
    bf16* kt = (bf16*)p.ktf + cg * 4 * DT * kFrag;
    constexpr int kQ = 4 * DT, kAll = kQ + (MODE == kDelta ? kQ : 0);
    for (int f = wave; f < kAll; f += 4) {
      const int fr = f < kQ ? f : f - kQ;
      const bf16* src = (f < kQ ? qs : ks) + ((fr / DT) * 16 + ln) * LS + (fr % DT) * 32 + g4;
      const bf16x4 x = *(const bf16x4*)src, y = *(const bf16x4*)(src + 16);
      bf16x8 o;
#pragma unroll
      for (int i = 0; i < 4; ++i) { o[i] = x[i]; o[4 + i] = y[i]; }
      *(bf16x8*)((f < kQ ? qf : kf) + fr * kFrag + lane * 8) = o;
    }
    for (int f = wave; f < kQ; f += 4) {
      const int d = (f >> 1) * 16 + ln, kb = f & 1;
      bf16x8 o;
#pragma unroll
      for (int e = 0; e < 8; ++e) o[e] = ks[(kb * 32 + 16 * (e >> 2) + g4 + (e & 3)) * LS + d];
      *(bf16x8*)(kt + f * kFrag + lane * 8) = o;
    }
  }
  if (MODE != kDelta) return;
  __syncthreads();
  // The inverse of I + A, by halves: both 32 x 32 diagonal blocks by forward substitution, a
  // column per lane of one wave (lanes 0 .. 31 the upper, 32 .. 63 the lower block), then the
  // lower left block as -T22 A21 T11.
  if (wave == 0) {
    const int o = lane & 32, col = lane & 31;
    float x[32];
#pragma unroll
    for (int i = 0; i < 32; ++i) {
      float a0 = col == i ? 1.f : 0.f, a1 = 0.f, a2 = 0.f, a3 = 0.f;
#pragma unroll
      for (int j = 0; j < i; j += 4) {
        const float4 a = *(const float4*)(am + (o + i) * AS + o + j);
        a0 = fmaf(-a.x, x[j], a0);
        if (j + 1 < i) a1 = fmaf(-a.y, x[j + 1], a1);
        if (j + 2 < i) a2 = fmaf(-a.z, x[j + 2], a2);
        if (j + 3 < i) a3 = fmaf(-a.w, x[j + 3], a3);
      }
      x[i] = (a0 + a1) + (a2 + a3);
    }
#pragma unroll
    for (int i = 0; i < 32; ++i) am[(o + i) * AS + o + col] = x[i];
  }
  __syncthreads();
  {
    constexpr int MS = 36;
    float* mid = (float*)qs;               // [32][MS]: q is not needed any more
    static_assert(kC * LS * sizeof(bf16) >= 32 * MS * sizeof(float), "the product fits q's rows");
    const int row = tid >> 3, c4 = (tid & 7) * 4;
    auto product = [&](const float* a, const float* b, int bs) {
      float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 8
      for (int j = 0; j < 32; ++j) {
        const float w = a[j];
        const float4 v = *(const float4*)(b + j * bs + c4);
        acc.x = fmaf(w, v.x, acc.x);
        acc.y = fmaf(w, v.y, acc.y);
        acc.z = fmaf(w, v.z, acc.z);
        acc.w = fmaf(w, v.w, acc.w);
      }
      return acc;
    };
    *(float4*)(mid + row * MS + c4) = product(am + (32 + row) * AS, am, AS);
    __syncthreads();
    const float4 t = product(am + (32 + row) * AS + 32, mid, MS);
    *(float4*)(am + (32 + row) * AS + c4) = make_float4(-t.x, -t.y, -t.z, -t.w);
  }
  __syncthreads();
  bf16* tf = (bf16*)p.tf + ch * kPT * kFrag;
  for (int f = wave; f < 6; f += 4) {
    const int tt = f < 2 ? f : 2 + ((f - 2) >> 1), kb = f < 2 ? 0 : (f - 2) & 1;
    const float* src = am + (tt * 16 + ln) * AS + kb * 32 + g4;
    const float4 x = *(const float4*)src, y = *(const float4*)(src + 16);
    const float v[8] = {x.x, x.y, x.z, x.w, y.x, y.y, y.z, y.w};
    bf16x8 vh, vl;
    split8(v, vh, vl);
    *(bf16x8*)(tf + f * kFrag + lane * 8) = vh;
    *(bf16x8*)(tf + (6 + f) * kFrag + lane * 8) = vl;
  }
}

// ------------------------------------------------------------------ walk over the chunks
// A workgroup per (sequence, head, NW x 16 state columns); a wave owns 16 columns.  The
// normaliser of the matrix memory is one more wave (of the head's first workgroup) whose single
// column has ones for values.  The operand fragments and scalars of a chunk go to LDS by
// LDS-DMA, one chunk ahead of the products where two chunks fit; the values of the next chunk are
// fetched into registers.
__device__ __forceinline__ void dma16(const void* g, void* lds_wave_base) {
  __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)g,
                                   (__attribute__((address_space(3))) void*)lds_wave_base, 16, 0, 0);
}

template <int MODE, int DT>
struct Walk {
  static constexpr int F = 4 * DT;                               // fragments of q, k, k transposed
  static constexpr int Q = 0;                                    // fragment indices in a buffer
  static constexpr int K = Q + F;
  static constexpr int P = K + (MODE == kDelta ? F : 0);
  static constexpr int T = P + kPT;
  static constexpr int KT = T + (MODE == kDelta ? kPT : 0);
  static constexpr int SC = KT + F;
  static constexpr int N = SC + 1;                               // 1 KB each
  static constexpr int NB = N <= 80 ? 2 : 1;                     // buffers (160 KB of LDS)
};

template <int MODE, int DT, int NW>
__global__ __launch_bounds__(NW * 64 + (MODE == kMatrixMemory ? 64 : 0)) void chunk_walk_kernel(
    ChunkParams p) {
  using W = Walk<MODE, DT>;
  constexpr int D = DT * 32;
  __shared__ __align__(16) bf16 lds[W::NB * W::N * kFrag];
  const RecurrenceParams& r = p.r;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int lane = threadIdx.x & 63, g4 = (lane >> 4) * 4, ln = lane & 15;
  const int nct = (r.V + NW * 16 - 1) / (NW * 16);
  // the workgroups of a sequence's heads share an XCD
  const int id = akap::xcd_remap(blockIdx.x, gridDim.x);
  const int h = (id / nct) % r.H, b = id / (nct * r.H), ct = id % nct;
  const int first = r.q_start[b], end = r.q_start[b + 1];
  if (end <= first) return;
  const int slot = r.seq_slot[first];
  if (slot < 0 || slot >= r.num_slots) return;
  const int rep = r.H / r.G, hq = h / rep;
  const bool nwave = MODE == kMatrixMemory && wave == NW;        // the normaliser's wave
  const int c0 = (ct * NW + wave) * 16, c = c0 + ln;
  const bool isv = !nwave && c < r.V, isn = nwave && ct == 0 && ln == 0;
  // wave-uniform: a wave past the columns only stages
  const bool active = nwave ? ct == 0 : c0 < r.V;
  float* sp = nwave ? r.n_state + ((size_t)slot * r.H + h) * D
                    : r.state + (((size_t)slot * r.H + h) * r.V + (isv ? c : 0)) * D;

  auto stage = [&](int entry, int buf) {
    if (MODE == kMatrixMemory && wave >= NW) return;
    const size_t ch = (size_t)entry * r.H + h, cg = (size_t)entry * r.G + hq;
    bf16* dst = lds + buf * W::N * kFrag;
    auto seg = [&](const uint16_t* src, int at, auto n) {
      static_assert(decltype(n)::value % 4 == 0, "whole rounds of four waves");
#pragma unroll
      for (int f = 0; f < decltype(n)::value; f += NW)
        if (decltype(n)::value % NW == 0 || f + wave < decltype(n)::value)
          dma16(src + (f + wave) * kFrag + lane * 8, dst + (at + f + wave) * kFrag);
    };
    using NF = std::integral_constant<int, W::F>;
    using NP = std::integral_constant<int, kPT>;
    if (MODE == kDelta) seg(p.kf + cg * W::F * kFrag, W::K, NF());
    seg(p.qf + cg * W::F * kFrag, W::Q, NF());
    if (MODE == kDelta) seg(p.tf + ch * kPT * kFrag, W::T, NP());
    seg(p.pf + ch * kPT * kFrag, W::P, NP());
    seg(p.ktf + cg * W::F * kFrag, W::KT, NF());
    if (wave == 0) dma16(p.sc + ch * kSc + lane * 4, dst + W::SC * kFrag);
  };
  // values of this lane's column, rows as in an accumulator, a register each: packing two would
  // wait for the loads (columns past V load column 0 and are masked at their use)
  const uint32_t vbytes = (uint32_t)(isv ? c : 0) * 2u;
  auto values = [&](int r0, uint32_t (&v)[16]) {
    const int n = min(kC, end - r0);
    const char* row0 = (const char*)((const uint16_t*)r.qkv + (size_t)r0 * r.qkv_stride + r.v_off +
                                     h * r.V);
    const uint32_t rb = (uint32_t)r.qkv_stride * 2u;
    if (n == kC) {
      const uint32_t lo = vbytes + (uint32_t)g4 * rb;
#pragma unroll
      for (int i = 0; i < 16; ++i)
        v[i] = *(const uint16_t*)(row0 + (size_t)((i >> 2) * 16 + (i & 3)) * rb + lo);
    } else {
#pragma unroll
      for (int i = 0; i < 16; ++i)
        v[i] = *(const uint16_t*)(row0 + (uint32_t)min((i >> 2) * 16 + g4 + (i & 3), n - 1) * rb +
                                  vbytes);
    }
  };

  f32x4 S[2 * DT];
  const bool carry = r.positions[first] != 0 && (isv || isn);
#pragma unroll
  for (int d = 0; d < 2 * DT; ++d) {
    float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
    if (carry) x = *(const float4*)(sp + d * 16 + g4);
    S[d] = f32x4{x.x, x.y, x.z, x.w};
  }
  int entry = chunk_base(r.q_start, b, p.row0);
  int buf = 0;
  const uint32_t vmask = isv ? 0xffffu : 0u, vone = isn ? 0x3f80u : 0u;   // bf16 1.0
  uint32_t nv[16];
  values(first, nv);
  if (W::NB == 2) stage(entry, 0);
  for (int r0 = first; r0 < end; r0 += kC, ++entry) {
    const int n = min(kC, end - r0);
    if (W::NB == 1) {
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      __builtin_amdgcn_s_barrier();       // every wave has read the previous chunk
      asm volatile("" ::: "memory");
      stage(entry, 0);
    }
    // a builtin wait (vmcnt 0, lgkmcnt 0): the compiler then knows that the values fetched during
    // the previous chunk have arrived, and adds no wait of its own after the next ones are issued
    __builtin_amdgcn_s_waitcnt(0x0070);
    asm volatile("" ::: "memory");
    __builtin_amdgcn_s_barrier();         // this chunk has landed; the other buffer is free
    asm volatile("" ::: "memory");
    const float eend = p.eend[(size_t)entry * r.H + h];
    float vv[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) vv[i] = __uint_as_float(((nv[i] & vmask) | vone) << 16);
    if (r0 + kC < end) {
      if (W::NB == 2) stage(entry + 1, buf ^ 1);
      values(r0 + kC, nv);
    }
    const bf16* cur = lds + buf * W::N * kFrag;
    if (W::NB == 2) buf ^= 1;
    if (!active) continue;
    const bf16* fl = cur + lane * 8;
    auto frag = [&](int i) { return *(const bf16x8*)(fl + i * kFrag); };
    // scalars of the four rows 16 t + 4 g .. +3 of array a
    const bf16* sl = cur + W::SC * kFrag + g4 * 2;
    auto sc4 = [&](int a, int t) {
      return __builtin_bit_cast(f32x4, *(const bf16x8*)(sl + (a * kC + t * 16) * 2));
    };
    if (MODE == kDecay && r.act) {
#pragma unroll
      for (int i = 0; i < 16; ++i) vv[i] *= sigmoidf(vv[i]);
    }
    // products with the state before the chunk
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    f32x4 O[4] = {zero, zero, zero, zero}, X[4] = {zero, zero, zero, zero};
#pragma unroll
    for (int k = 0; k < DT; ++k) {
      float s[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) s[e] = S[2 * k + (e >> 2)][e & 3];
      bf16x8 sh, sl2;
      split8(s, sh, sl2);
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        if (MODE == kDelta) {
          const bf16x8 a = frag(W::K + t * DT + k);
          X[t] = mfma(a, sh, X[t]);
          X[t] = mfma(a, sl2, X[t]);
        }
        const bf16x8 a = frag(W::Q + t * DT + k);
        O[t] = mfma(a, sh, O[t]);
        O[t] = mfma(a, sl2, O[t]);
      }
    }
    if (MODE == kDelta) {
      // u = (I + A)^-1 (beta v - beta e^L c (K S0))
      bf16x8 xh[2], xl[2];
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        float x[8];
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          const f32x4 be = sc4(2, 2 * kb + i), bk = sc4(3, 2 * kb + i);
#pragma unroll
          for (int j = 0; j < 4; ++j)
            x[4 * i + j] = be[j] * vv[kb * 8 + 4 * i + j] - bk[j] * X[2 * kb + i][j];
        }
        split8(x, xh[kb], xl[kb]);
      }
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        X[t] = zero;
#pragma unroll
        for (int kb = 0; kb <= t >> 1; ++kb) {
          const bf16x8 ah = frag(W::T + tri(t, kb)), al = frag(W::T + 6 + tri(t, kb));
          X[t] = mfma(ah, xh[kb], X[t]);
          X[t] = mfma(ah, xl[kb], X[t]);
          X[t] = mfma(al, xh[kb], X[t]);
        }
      }
    }
    // outputs: the part through S0 scaled by row, the part inside the chunk
#pragma unroll
    for (int t = 0; t < 4; ++t) O[t] *= sc4(0, t);
    bf16x8 wh[2], wl[2];        // what enters the state: hi + lo of e^(L_end - L) c x
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      bf16x8 uh, ul;
      float u[8], w[8];
#pragma unroll
      for (int e = 0; e < 8; ++e)
        u[e] = MODE == kDelta ? X[2 * kb + (e >> 2)][e & 3] : vv[kb * 8 + e];
      // (plain recurrences: v is a bf16 number or, activated, rounded to one by its lo part)
      split8(u, uh, ul);
#pragma unroll
      for (int t = 2 * kb; t < 4; ++t) {
        const bf16x8 ah = frag(W::P + tri(t, kb)), al = frag(W::P + 6 + tri(t, kb));
        O[t] = mfma(ah, uh, O[t]);
        O[t] = mfma(al, uh, O[t]);
        if (MODE != kMatrixMemory) O[t] = mfma(ah, ul, O[t]);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const f32x4 z = sc4(1, 2 * kb + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) w[4 * i + j] = u[4 * i + j] * z[j];
      }
      split8(w, wh[kb], wl[kb]);
    }
    {
      const size_t os = (nwave ? (size_t)r.H : (size_t)r.H * r.V) * sizeof(float);   // row pitch
      char* o = nwave ? (char*)(p.den + (size_t)r0 * r.H + h)
                      : (char*)(r.raw + ((size_t)r0 * r.H + h) * r.V);
      const uint32_t lo = (uint32_t)(nwave ? 0 : c) * 4u + (uint32_t)g4 * (uint32_t)os;
      if (isv || isn) {
        if (n == kC) {
#pragma unroll
          for (int i = 0; i < 16; ++i)
            *(float*)(o + ((i >> 2) * 16 + (i & 3)) * os + lo) = O[i >> 2][i & 3];
        } else {
#pragma unroll
          for (int i = 0; i < 16; ++i)
            if ((i >> 2) * 16 + g4 + (i & 3) < n)
              *(float*)(o + ((i >> 2) * 16 + (i & 3)) * os + lo) = O[i >> 2][i & 3];
        }
      }
    }
    // the state after the chunk
#pragma unroll
    for (int d = 0; d < 2 * DT; ++d) {
      S[d] *= eend;
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        const bf16x8 a = frag(W::KT + d * 2 + kb);
        S[d] = mfma(a, wh[kb], S[d]);
        S[d] = mfma(a, wl[kb], S[d]);
      }
    }
  }
  if (isv || isn) {
#pragma unroll
    for (int d = 0; d < 2 * DT; ++d)
      *(float4*)(sp + d * 16 + g4) = make_float4(S[d][0], S[d][1], S[d][2], S[d][3]);
  }
}

// ------------------------------------------------------------------ gates of the matrix memory
// a wave per (sequence, head), 64 tokens a turn: the running maximum m_t = max(f_t + m_(t-1), i_t)
// is a scan over the maps m -> max(F + m, I), composed by lane exchange
__global__ __launch_bounds__(64) void memory_gates_kernel(ChunkParams p) {
  const RecurrenceParams& r = p.r;
  const int b = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int first = r.q_start[b], end = r.q_start[b + 1];
  if (end <= first) return;
  const int slot = r.seq_slot[first];
  if (slot < 0 || slot >= r.num_slots) return;
  float* ms = r.m_state + (size_t)slot * r.H + h;
  float m = r.positions[first] == 0 ? 0.f : *ms;
  const float fb = r.pa[h], ib = r.pb[h], icap = 1.0f / r.cap;
  auto fetch = [&](int row, bf16& f, bf16& i) {
    const bf16* pr = (const bf16*)r.proj + (size_t)min(row, end - 1) * r.proj_stride;
    f = pr[r.a_off + h];
    i = pr[r.b_off + h];
  };
  bf16 nf, ni;                         // the next 64 tokens' inputs, in flight
  fetch(first + lane, nf, ni);
  for (int r0 = first; r0 < end; r0 += 64) {
    const int row = r0 + lane;
    const bool live = row < end;
    float f = 0.f, i = -INFINITY;      // past the end: the identity
    const float zf = (float)nf, zi = (float)ni;
    fetch(row + 64, nf, ni);
    if (live) {
      f = -softplusf(-r.cap * tanhf((zf + fb) * icap));
      i = r.cap * tanhf((zi + ib) * icap);
    }
    float F = f, I = i;
    for (int o = 1; o < 64; o <<= 1) {
      const float Fp = __shfl_up(F, o, 64), Ip = __shfl_up(I, o, 64);
      if (lane >= o) {
        I = fmaxf(F + Ip, I);
        F += Fp;
      }
    }
    const float mt = fmaxf(F + m, I);
    float mp = __shfl_up(mt, 1, 64);
    if (lane == 0) mp = m;
    if (live) {
      const size_t at = (size_t)row * r.H + h;
      p.la[at] = f + mp - mt;
      p.lb[at] = expf(i - mt);
      p.floor[at] = expf(-mt);
    }
    m = __shfl(mt, 63, 64);
  }
  if (lane == 0) *ms = m;
}

}  // namespace

// ================================================================== launchers
bool chunk_supported(int D) { return D == 32 || D == 64 || D == 96 || D == 128 || D == 256; }

// bf16 elements / floats of a workspace of `chunks` chunk entries
void chunk_workspace(int mode, int chunks, int H, int G, int D, int64_t* halves, int64_t* floats) {
  const int64_t g = (int64_t)chunks * G, hh = (int64_t)chunks * H;
  *halves = g * (int64_t)(D / 16) * 2 * kFrag * (mode == kDelta ? 2 : 1) +
            g * (D / 32) * 4 * kFrag + hh * kPT * kFrag * (mode == kDelta ? 2 : 1);
  *floats = hh * (kSc + 1);
}

void launch_chunk_recurrence(ChunkParams p, int mode, uint16_t* halves, float* floats,
                             hipStream_t s) {
  const RecurrenceParams& r = p.r;
  if (r.num_seqs <= 0 || p.num_chunks <= 0) return;
  const int64_t g = (int64_t)p.num_chunks * r.G, hh = (int64_t)p.num_chunks * r.H;
  const int64_t rows = g * (r.D / 16) * 2 * kFrag;
  uint16_t* w = halves;
  p.qf = w; w += rows;
  p.kf = w;
  if (mode == kDelta) w += rows;
  p.ktf = w; w += g * (r.D / 32) * 4 * kFrag;
  p.pf = w; w += hh * kPT * kFrag;
  p.tf = w;
  p.sc = floats;
  p.eend = floats + hh * kSc;
  const dim3 pg(p.num_chunks, r.H);
  // workgroups of eight waves share a staged chunk among 128 columns; of four when those would
  // leave CUs idle
  const int wg8 = (r.V + 127) / 128 * r.H * r.num_seqs, wg4 = (r.V + 63) / 64 * r.H * r.num_seqs;
  const bool eight = wg8 >= 256;
  const int extra = mode == kMatrixMemory ? 64 : 0;
  if (mode == kMatrixMemory) memory_gates_kernel<<<dim3(r.num_seqs, r.H), 64, 0, s>>>(p);
#define AKAP_CH(M, T)                                \
  do {                                               \
    chunk_prep_kernel<M, T><<<pg, 256, 0, s>>>(p);   \
    if (eight) chunk_walk_kernel<M, T, 8><<<wg8, 512 + extra, 0, s>>>(p);   \
    else chunk_walk_kernel<M, T, 4><<<wg4, 256 + extra, 0, s>>>(p);         \
  } while (0)
#define AKAP_CHD(M)                    \
  switch (r.D / 32) {                  \
    case 1: AKAP_CH(M, 1); break;      \
    case 2: AKAP_CH(M, 2); break;      \
    case 3: AKAP_CH(M, 3); break;      \
    case 4: AKAP_CH(M, 4); break;      \
    default: AKAP_CH(M, 8); break;     \
  }
  if (mode == kDecay) AKAP_CHD(kDecay)
  else if (mode == kMatrixMemory) AKAP_CHD(kMatrixMemory)
  else AKAP_CHD(kDelta)
#undef AKAP_CHD
#undef AKAP_CH
}

}  // namespace akap_stream
