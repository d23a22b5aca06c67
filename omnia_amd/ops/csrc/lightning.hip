// Linear attention with one fixed decay per head (lightning attention) for gfx950: a
// [dim x vdim] fp32 state per sequence and head,
//
//     S <- a S + k v^T ;  o = S^T q ;  q, k, v = silu of projections
//
// and behind it one RMS norm over all heads together and a sigmoid output gate.  One fused
// input projection feeds it, a row of [q (H*Dp) | k (H*Dp) | v (H*Vp) | g (H*Vp)], head
// widths padded with zeros to multiples of 8.
//
//   lightning_step   decode: one token per sequence, one workgroup per (row, head)
//   lightning_scan   prefill: each sequence's new tokens in segments of L.  With a fixed
//                    decay the state a segment adds depends on nothing before it, so
//                    1 scan_kernel<.., false>: every segment's own state, from zeros
//                    2 chain_kernel: the states the segments start from, a^L apart
//                    3 scan_kernel<.., true>: outputs of every segment from its start state
//                    all segments at once; portions of up to L tokens need step 3 only.
//                    Wide heads take a token-by-token kernel instead
//   lightning_norm   norm and gate of the outputs of either
//
// State of sequence slot s: state[s][h][Dp][Vp] fp32.  A sequence whose first row of this
// launch is at position 0 starts from zeros, whatever its slot held: slots are never
// cleared.  A negative slot (padded graph row) reads and writes no state.  Everything in
// the recurrence is fp32.  The products of fp32 models are fp32 MFMA; bf16 models round q,
// k and v to bf16 and split every fp32 operand (state, decayed scores and values) into
// three bf16 parts that hold all its bits, so that bf16 MFMA multiplies it unrounded.
#include "common.h"

using namespace omnia;

namespace {

constexpr int kPow = 48;     // a row of the power table: a^0 .. a^32, then a^(64 * 2^i)
constexpr int kPowSeg = 33;  // first of the latter

// projection rows or their split-K slabs
struct Src {
  const void* p;
  int type, S;  // storage 0 bf16, 1 fp32, 2 fp16
  int64_t ld, slab;
  __device__ __forceinline__ float one(int64_t i) const {
    return type == 1 ? ((const float*)p)[i]
                     : type == 2 ? (float)((const _Float16*)p)[i] : bf2f(((const bf16_t*)p)[i]);
  }
  // four neighbouring columns (c % 4 == 0)
  __device__ __forceinline__ float4v four(int64_t i) const {
    if (type == 1) return *reinterpret_cast<const float4v*>((const float*)p + i);
    if (type == 2) {
      typedef _Float16 half4v __attribute__((ext_vector_type(4)));
      const half4v h = *reinterpret_cast<const half4v*>((const _Float16*)p + i);
      return float4v{(float)h[0], (float)h[1], (float)h[2], (float)h[3]};
    }
    const short4v h = *reinterpret_cast<const short4v*>((const bf16_t*)p + i);
    return float4v{bf2f((uint16_t)h[0]), bf2f((uint16_t)h[1]), bf2f((uint16_t)h[2]),
                   bf2f((uint16_t)h[3])};
  }
  __device__ __forceinline__ float4v at4(int t, int c) const {
    const int64_t i = (int64_t)t * ld + c;
    float4v v = four(i);
    for (int s = 1; s < S; s += 4) {
      float4v q[4];
#pragma unroll
      for (int j = 0; j < 4; ++j)
        q[j] = s + j < S ? four(i + (s + j) * slab) : float4v{0.f, 0.f, 0.f, 0.f};
      v += (q[0] + q[1]) + (q[2] + q[3]);
    }
    return v;
  }
  __device__ __forceinline__ float at(int t, int c) const {
    const int64_t i = (int64_t)t * ld + c;
    float v = one(i);
    for (int s = 1; s < S; s += 4) {  // four slabs in flight
      float q[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) q[j] = s + j < S ? one(i + (s + j) * slab) : 0.f;
      v += (q[0] + q[1]) + (q[2] + q[3]);
    }
    return v;
  }
};

__device__ __forceinline__ float4v silu4(float4v v) {
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] = siluf_(v[j]);
  return v;
}

__device__ __forceinline__ float4v mfma4(float a, float b, float4v c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// -------------------------------------------------------------- lightning_step
// grid (rows, H), 256 threads.  Thread (cg, rg): 4 state columns cg*4.., the rows
// rg, rg + RG, ... kept in registers (NR of them).
template <int NR>
__global__ __launch_bounds__(256) void step_kernel(float* __restrict__ o,
                                                   float* __restrict__ state, Src x,
                                                   const float* __restrict__ pw,
                                                   const int* __restrict__ positions,
                                                   const int* __restrict__ slots, int H, int Dp,
                                                   int Vp) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int slot = slots[t];
  float* orow = o + ((int64_t)t * H + h) * Vp;
  if (slot < 0) {
    for (int i = tid; i < Vp; i += 256) orow[i] = 0.f;
    return;
  }
  const bool fresh = positions[t] == 0;
  const int CG = Vp / 4, RG = 256 / CG;
  float* qs = sm;        // [Dp]
  float* ks = qs + Dp;   // [Dp]
  float* vs = ks + Dp;   // [Vp]
  float* red = vs + Vp;  // [RG][Vp]
  const int cg = tid % CG, rg = tid / CG;
  const bool act = rg < RG;
  float4v* S = reinterpret_cast<float4v*>(state + ((int64_t)slot * H + h) * Dp * Vp) + cg;
  float4v reg[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int d = rg + i * RG;
    reg[i] = (act && d < Dp && !fresh) ? S[(int64_t)d * CG] : float4v{0.f, 0.f, 0.f, 0.f};
  }
  const float a = pw[h * kPow + 1];
  for (int i = tid * 4; i < 2 * Dp + Vp; i += 1024) {  // q | k | v of this head
    const int c = i < 2 * Dp ? (i < Dp ? h * Dp + i : H * Dp + h * Dp + i - Dp)
                             : 2 * H * Dp + h * Vp + i - 2 * Dp;
    *reinterpret_cast<float4v*>(sm + i) = silu4(x.at4(t, c));
  }
  __syncthreads();
  float4v acc = {0.f, 0.f, 0.f, 0.f};
  if (act) {
    const float4v v4 = *reinterpret_cast<const float4v*>(vs + cg * 4);
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int d = rg + i * RG;
      if (d < Dp) {
        reg[i] = reg[i] * a + v4 * ks[d];
        acc += reg[i] * qs[d];
        S[(int64_t)d * CG] = reg[i];
      }
    }
    *reinterpret_cast<float4v*>(red + rg * Vp + cg * 4) = acc;
  }
  __syncthreads();
  for (int j = tid; j < Vp; j += 256) {
    float v = 0.f;
    for (int r = 0; r < RG; ++r) v += red[r * Vp + j];
    orow[j] = v;
  }
}

// any head sizes: grid (H, sequences), a thread per state column, the state in place.
// q_start null: one row per sequence.
__global__ __launch_bounds__(256) void any_kernel(float* __restrict__ o,
                                                  float* __restrict__ state, Src x,
                                                  const float* __restrict__ pw,
                                                  const int* __restrict__ q_start,
                                                  const int* __restrict__ positions,
                                                  const int* __restrict__ slots, int H, int Dp,
                                                  int Vp) {
  extern __shared__ float sm[];  // q [Dp] | k [Dp]
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int row0 = q_start ? q_start[s] : s, n = q_start ? q_start[s + 1] - row0 : 1;
  const int slot = slots[s];
  if (n <= 0) return;
  if (slot < 0) {
    for (int i = tid; i < n * Vp; i += 256)
      o[((int64_t)(row0 + i / Vp) * H + h) * Vp + i % Vp] = 0.f;
    return;
  }
  const bool fresh = positions[row0] == 0;
  const float a = pw[h * kPow + 1];
  float* S = state + ((int64_t)slot * H + h) * Dp * Vp;
  for (int t = row0; t < row0 + n; ++t) {
    __syncthreads();
    for (int i = tid; i < 2 * Dp; i += 256)
      sm[i] = siluf_(x.at(t, i < Dp ? h * Dp + i : H * Dp + h * Dp + i - Dp));
    __syncthreads();
    for (int j = tid; j < Vp; j += 256) {
      const float v = siluf_(x.at(t, 2 * H * Dp + h * Vp + j));
      float acc = 0.f;
      for (int d = 0; d < Dp; ++d) {
        const float old = fresh && t == row0 ? 0.f : S[(int64_t)d * Vp + j];
        const float nw = a * old + sm[Dp + d] * v;
        S[(int64_t)d * Vp + j] = nw;
        acc += nw * sm[d];
      }
      o[((int64_t)t * H + h) * Vp + j] = acc;
    }
  }
}

// -------------------------------------------------------------- lightning_scan
// Within a block of 16 tokens, S0 the state before it:
//     o_t = a^(t+1) S0^T q_t + sum_{i<=t} a^(t-i) (q_t . k_i) v_i
//     S   = a^m S0 + sum_i a^(m-1-i) k_i v_i^T          (m tokens, 16 but in the last block)
// Rows past the end have k = 0 and weight 0.
//
// segment j of sequence s has number seg_base(s) + j: leaves room for every earlier
// sequence's ragged segment
__device__ __forceinline__ int seg_base(const int* q_start, int s, int L) {
  return q_start[s] / L + s;
}

template <typename T>
struct Raw4;
template <>
struct Raw4<bf16_t> {
  typedef short4v type;
  static __device__ __forceinline__ float4v f(short4v h) {
    return float4v{bf2f((uint16_t)h[0]), bf2f((uint16_t)h[1]), bf2f((uint16_t)h[2]),
                   bf2f((uint16_t)h[3])};
  }
};
template <>
struct Raw4<float> {
  typedef float4v type;
  static __device__ __forceinline__ float4v f(float4v h) { return h; }
};
struct Scan {
  float* o;       // [T][H][Vp]
  float* state;   // [slots][H][Dp][Vp]
  float* seg;     // [segments][H][Dp][Vp]
  const float* pw;
  const int* q_start;
  const int* positions;
  const int* slots;
  int64_t ldx;
  int nseq, H, Dp, Vp, L;
};

// grid (segments, H, column groups of 64 NC), 4 waves; wave w owns the NC column tiles
// 16 (w NC + c) of its group, its part of the state as ND x NC accumulator tiles (key
// dimensions 16 j + 4 (lane >> 4) + r in register r).  The accumulator layout serves as the
// B operand of the next product as it stands: k-step r takes dimension (token)
// 4 (lane >> 4) + r, and the A side is read in that order.  32 tokens a step.
template <typename T, int ND, int NC, bool OUT>
__global__ __launch_bounds__(256, ND <= 8 ? 2 : 1) void scan_kernel(const T* __restrict__ x,
                                                                   Scan p) {
  constexpr int DW = 16 * ND, KS = DW + 4, PS = 20;
  constexpr int NL = 32 * DW / 4 / 256;  // 4-element chunks a thread holds of 32 rows
  __shared__ __attribute__((aligned(16))) float kb[32 * KS];
  __shared__ __attribute__((aligned(16))) float qb[OUT ? 32 * KS : 4];
  __shared__ __attribute__((aligned(16))) float pb[OUT ? 4 * 16 * PS : 4];
  typedef typename Raw4<T>::type raw;
  const int id = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  int lo = 0, hi = p.nseq - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (seg_base(p.q_start, mid, p.L) <= id) lo = mid; else hi = mid - 1;
  }
  const int j0 = (id - seg_base(p.q_start, lo, p.L)) * p.L;
  const int all = p.q_start[lo + 1] - p.q_start[lo], n = min(p.L, all - j0);
  const int slot = p.slots[lo];
  const bool last = j0 + p.L >= all;
  if (n <= 0 || (!OUT && (last || slot < 0))) return;
  const int row0 = p.q_start[lo] + j0;
  const int lane = tid & 63, w = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int Dp = p.Dp, Vp = p.Vp, H = p.H;
  const int col0 = (blockIdx.z * 4 + w) * 16 * NC + c16;
  const float* pw = p.pw + h * kPow;

  float4v S[ND][NC];
  {
    const float* from = nullptr;
    if (OUT && slot >= 0) {
      if (all > p.L) from = p.seg + ((int64_t)id * H + h) * Dp * Vp;
      else if (p.positions[row0] != 0) from = p.state + ((int64_t)slot * H + h) * Dp * Vp;
    }
#pragma unroll
    for (int j = 0; j < ND; ++j)
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = 16 * j + 4 * g4 + r, col = col0 + 16 * c;
          S[j][c][r] = (from && d < Dp && col < Vp) ? from[(int64_t)d * Vp + col] : 0.f;
        }
  }
  // decays of this lane's places: a^(t+1) and, of a whole block, a^(15-t), t = 4 g4 + r
  float4v G, E;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    G[r] = pw[4 * g4 + r + 1];
    E[r] = pw[15 - 4 * g4 - r];
  }
  const float a16 = pw[16];

  const T* kx = x + (int64_t)row0 * p.ldx + (int64_t)H * Dp + h * Dp;
  const T* qx = x + (int64_t)row0 * p.ldx + h * Dp;
  const T* vx = x + (int64_t)row0 * p.ldx + (int64_t)2 * H * Dp + h * Vp;
  raw kreg[NL], qreg[OUT ? NL : 1];
  T vreg[2][NC][4];
  // Loads are unconditional: rows past the end re-read the last one (zeroed when they are
  // stored, or weighted with 0), columns past the head re-read its last ones.
  auto gload = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int e = i * 256 + tid, tt = min(t0 + e / (DW / 4), n - 1);
      const int64_t at = (int64_t)tt * p.ldx + min(e % (DW / 4) * 4, Dp - 4);
      kreg[i] = *reinterpret_cast<const raw*>(kx + at);
      if (OUT) qreg[i] = *reinterpret_cast<const raw*>(qx + at);
    }
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const T* vr = vx + (int64_t)min(t0 + 16 * b + 4 * g4 + r, n - 1) * p.ldx;
#pragma unroll
        for (int c = 0; c < NC; ++c) vreg[b][c][r] = vr[min(col0 + 16 * c, Vp - 1)];
      }
  };
  gload(0);
  for (int t0 = 0; t0 < n; t0 += 32) {
    __syncthreads();  // the previous tokens' LDS reads are done
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int e = i * 256 + tid, tt = e / (DW / 4), d4 = e % (DW / 4) * 4;
      const float4v z = {0.f, 0.f, 0.f, 0.f};
      const bool in = d4 < Dp && t0 + tt < n;
      *reinterpret_cast<float4v*>(kb + tt * KS + d4) = in ? silu4(Raw4<T>::f(kreg[i])) : z;
      if (OUT)
        *reinterpret_cast<float4v*>(qb + tt * KS + d4) = in ? silu4(Raw4<T>::f(qreg[i])) : z;
    }
    float4v v[2][NC];
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const bool in = t0 + 16 * b + 4 * g4 + r < n && col0 + 16 * c < Vp;
          v[b][c][r] = in ? siluf_(ldf(&vreg[b][c][r])) : 0.f;
        }
    __syncthreads();
    if (t0 + 32 < n) gload(t0 + 32);
    if constexpr (OUT) {
      // wave w: half (w & 1) of the key dimensions of block w >> 1's q k^T
      const float* qr = qb + (16 * (w >> 1) + c16) * KS + 4 * g4;
      const float* kr = kb + (16 * (w >> 1) + c16) * KS + 4 * g4;
      float4v s[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
      for (int jj = 0; jj < ND / 2; ++jj) {
        const int j = (w & 1) * (ND / 2) + jj;
        const float4v qa = *reinterpret_cast<const float4v*>(qr + 16 * j);
        const float4v ka = *reinterpret_cast<const float4v*>(kr + 16 * j);
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r & 1] = mfma4(qa[r], ka[r], s[r & 1]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {  // row t = 4 g4 + r, column i = c16
        const int t = 4 * g4 + r;
        pb[w * 16 * PS + t * PS + c16] = t >= c16 ? (s[0][r] + s[1][r]) * pw[t - c16] : 0.f;
      }
      __syncthreads();
    }
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const int m = n - t0 - 16 * b;
      if (m <= 0) break;
      const float* k0 = kb + 16 * b * KS;
      if constexpr (OUT) {
        float4v qs[NC][2];
#pragma unroll
        for (int c = 0; c < NC; ++c) qs[c][0] = qs[c][1] = float4v{0.f, 0.f, 0.f, 0.f};
        const float* q0 = qb + (16 * b + c16) * KS + 4 * g4;
#pragma unroll
        for (int j = 0; j < ND; ++j) {
          const float4v qa = *reinterpret_cast<const float4v*>(q0 + 16 * j);
#pragma unroll
          for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int c = 0; c < NC; ++c) qs[c][r & 1] = mfma4(qa[r], S[j][c][r], qs[c][r & 1]);
        }
        const float* p0 = pb + 2 * b * 16 * PS + c16 * PS + 4 * g4;
        const float4v pa = *reinterpret_cast<const float4v*>(p0) +
                           *reinterpret_cast<const float4v*>(p0 + 16 * PS);
        float4v ov[NC];
#pragma unroll
        for (int c = 0; c < NC; ++c) ov[c] = G * (qs[c][0] + qs[c][1]);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int c = 0; c < NC; ++c) ov[c] = mfma4(pa[r], v[b][c][r], ov[c]);
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          const int col = col0 + 16 * c;
          if (col < Vp) {
            float* op = p.o + ((int64_t)(row0 + t0 + 16 * b + 4 * g4) * H + h) * Vp + col;
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (4 * g4 + r < m) op[(int64_t)r * H * Vp] = ov[c][r];
          }
        }
      }
      float4v e = E;
      float am = a16;
      if (m < 16) {
        am = pw[m];
#pragma unroll
        for (int r = 0; r < 4; ++r) e[r] = 4 * g4 + r < m ? pw[m - 1 - 4 * g4 - r] : 0.f;
      }
#pragma unroll
      for (int c = 0; c < NC; ++c) v[b][c] *= e;
      // two key tiles at a time: independent products between dependent ones
#pragma unroll
      for (int j = 0; j < ND; j += 2) {
        float ka[2][4];
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
          for (int r = 0; r < 4; ++r) ka[i][r] = k0[(4 * g4 + r) * KS + 16 * (j + i) + c16];
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
          for (int c = 0; c < NC; ++c) S[j + i][c] *= am;
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int c = 0; c < NC; ++c) S[j + i][c] = mfma4(ka[i][r], v[b][c][r], S[j + i][c]);
      }
    }
  }
  if (slot < 0 || (OUT && !last)) return;
  float* to = OUT ? p.state + ((int64_t)slot * H + h) * Dp * Vp
                  : p.seg + ((int64_t)id * H + h) * Dp * Vp;
#pragma unroll
  for (int j = 0; j < ND; ++j)
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * j + 4 * g4 + r, col = col0 + 16 * c;
        if (d < Dp && col < Vp) to[(int64_t)d * Vp + col] = S[j][c][r];
      }
}

// ------------------------------------------- the same scan on bf16 MFMA (bf16 models)
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
__device__ __forceinline__ float4v mfma16(short8 a, short8 b, float4v c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                 __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
// eight fp32 values as three bf16 parts of 8 bits each (their sum is the value)
struct Split {
  short8 part[3];
};
__device__ __forceinline__ Split split8(float4v lo, float4v hi) {
  Split s;
#pragma unroll
  for (int k = 0; k < 3; ++k)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const uint32_t a = __float_as_uint(lo[j]), b = __float_as_uint(hi[j]);
      s.part[k][j] = (short)(a >> 16);
      s.part[k][4 + j] = (short)(b >> 16);
      lo[j] -= __uint_as_float(a & 0xffff0000u);
      hi[j] -= __uint_as_float(b & 0xffff0000u);
    }
  return s;
}

// As scan_kernel, 32 tokens a block, two LDS buffers and one barrier a block.  Products
// over 32 key dimensions (or tokens) take, in lane group g4 = lane >> 4, the dimensions
// 4 g4 + r of one 16-tile and of the next (r < 4): what the state's accumulators hold.  The
// scores are made transposed (row i, column t), which is the A operand of P V as it stands.
template <int ND, int NC, bool OUT>
__global__ __launch_bounds__(256, ND <= 8 ? 2 : 1) void scan16_kernel(const bf16_t* __restrict__ x, Scan p) {
  constexpr int DW = 16 * ND, KS = DW + 8, NJ = ND / 2;
  constexpr int NL = 32 * DW / 4 / 256;
  struct Buf {
    bf16_t k[32 * KS], q[OUT ? 32 * KS : 8];
  };
  __shared__ __attribute__((aligned(16))) Buf buf[2];
  const int id = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  int lo = 0, hi = p.nseq - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (seg_base(p.q_start, mid, p.L) <= id) lo = mid; else hi = mid - 1;
  }
  const int j0 = (id - seg_base(p.q_start, lo, p.L)) * p.L;
  const int all = p.q_start[lo + 1] - p.q_start[lo], n = min(p.L, all - j0);
  const int slot = p.slots[lo];
  const bool last = j0 + p.L >= all;
  if (n <= 0 || (!OUT && (last || slot < 0))) return;
  const int row0 = p.q_start[lo] + j0;
  const int lane = tid & 63, w = tid >> 6, c16 = lane & 15, g4 = lane >> 4;
  const int Dp = p.Dp, Vp = p.Vp, H = p.H;
  const int col0 = (blockIdx.z * 4 + w) * 16 * NC + c16;
  const float* pw = p.pw + h * kPow;
  const float4v zero = {0.f, 0.f, 0.f, 0.f};

  float4v S[ND][NC];
  {
    const float* from = nullptr;
    if (OUT && slot >= 0) {
      if (all > p.L) from = p.seg + ((int64_t)id * H + h) * Dp * Vp;
      else if (p.positions[row0] != 0) from = p.state + ((int64_t)slot * H + h) * Dp * Vp;
    }
#pragma unroll
    for (int j = 0; j < ND; ++j)
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = 16 * j + 4 * g4 + r, col = col0 + 16 * c;
          S[j][c][r] = (from && d < Dp && col < Vp) ? from[(int64_t)d * Vp + col] : 0.f;
        }
  }
  // decays of this lane's places: outputs a^(t+1) and values a^(31-t) at t = 4 g4 + r (+ 16),
  // scores a^(t-i) at t = c16, i = 4 g4 + r of one tile and of the one before
  float4v G[2], E[2], Pd, Po;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = 4 * g4 + r;
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      G[b][r] = pw[16 * b + t + 1];
      E[b][r] = pw[31 - 16 * b - t];
    }
    Pd[r] = c16 >= t ? pw[max(c16 - t, 0)] : 0.f;
    Po[r] = pw[16 + c16 - t];
  }
  const float a32 = pw[32];

  const bf16_t* kx = x + (int64_t)row0 * p.ldx + (int64_t)H * Dp + h * Dp;
  const bf16_t* qx = x + (int64_t)row0 * p.ldx + h * Dp;
  const bf16_t* vx = x + (int64_t)row0 * p.ldx + (int64_t)2 * H * Dp + h * Vp;
  short4v kreg[NL], qreg[OUT ? NL : 1];
  bf16_t vreg[2][NC][4];
  // unconditional loads: rows past the end re-read the last one, columns past the head its
  // last ones (zeroed when they are used)
  auto gload = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int e = i * 256 + tid, tt = min(t0 + e / (DW / 4), n - 1);
      const int64_t at = (int64_t)tt * p.ldx + min(e % (DW / 4) * 4, Dp - 4);
      kreg[i] = *reinterpret_cast<const short4v*>(kx + at);
      if (OUT) qreg[i] = *reinterpret_cast<const short4v*>(qx + at);
    }
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const bf16_t* vr = vx + (int64_t)min(t0 + 16 * b + 4 * g4 + r, n - 1) * p.ldx;
#pragma unroll
        for (int c = 0; c < NC; ++c) vreg[b][c][r] = vr[min(col0 + 16 * c, Vp - 1)];
      }
  };
  auto lwrite = [&](Buf& B, int t0) {
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int e = i * 256 + tid, tt = e / (DW / 4), d4 = e % (DW / 4) * 4;
      const bool in = d4 < Dp && t0 + tt < n;
      auto put = [&](bf16_t* to, short4v v) {
        const float4v f = silu4(Raw4<bf16_t>::f(v));
        uint2v o;
        o[0] = in ? pack_bf2(f[0], f[1]) : 0u;
        o[1] = in ? pack_bf2(f[2], f[3]) : 0u;
        *reinterpret_cast<uint2v*>(to + tt * KS + d4) = o;
      };
      put(B.k, kreg[i]);
      if constexpr (OUT) put(B.q, qreg[i]);
    }
  };
  typedef short v4s __attribute__((ext_vector_type(4)));
  typedef __attribute__((address_space(3))) v4s* lds_v4s;
  auto frag = [&](const bf16_t* base, int tile, int jj) {  // rows of a tile, 32 dimensions
    const bf16_t* at = base + (16 * tile + c16) * KS + 32 * jj + 4 * g4;
    return __builtin_shufflevector(*reinterpret_cast<const v4s*>(at),
                                   *reinterpret_cast<const v4s*>(at + 16), 0, 1, 2, 3, 4, 5, 6, 7);
  };

  gload(0);
  lwrite(buf[0], 0);
  const int nblk = (n + 31) / 32;
  for (int bi = 0; bi < nblk; ++bi) {
    const int t0 = 32 * bi, m = n - t0;
    Buf& B = buf[bi & 1];
    short8 vb[NC];  // values at tokens 4 g4 + r (+ 16)
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const bool in = 16 * b + 4 * g4 + r < m && col0 + 16 * c < Vp;
          vb[c][4 * b + r] = in ? (short)f2bf(siluf_(bf2f(vreg[b][c][r]))) : (short)0;
        }
    // this block's operands are complete, and every wave is done with the other buffer
    __syncthreads();
    if (bi + 1 < nblk) gload(t0 + 32);
    if constexpr (OUT) {
      float4v s00 = zero, s10 = zero, s11 = zero;  // scores of (t tile, i tile), transposed
#pragma unroll
      for (int jj = 0; jj < NJ; ++jj) {
        const short8 k0 = frag(B.k, 0, jj), k1 = frag(B.k, 1, jj);
        const short8 q0 = frag(B.q, 0, jj), q1 = frag(B.q, 1, jj);
        s00 = mfma16(k0, q0, s00);
        s10 = mfma16(k0, q1, s10);
        s11 = mfma16(k1, q1, s11);
      }
      __builtin_amdgcn_sched_barrier(0);  // registers: the scores first
      const Split p0 = split8(s00 * Pd, zero), p1 = split8(s10 * Po, s11 * Pd);
      float4v o[2][NC];
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int c = 0; c < NC; ++c) o[b][c] = zero;
#pragma unroll
      for (int jj = 0; jj < NJ; ++jj) {
        const short8 qf[2] = {frag(B.q, 0, jj), frag(B.q, 1, jj)};
#pragma unroll
        for (int c = 0; c < NC; ++c) {
          const Split st = split8(S[2 * jj][c], S[2 * jj + 1][c]);
#pragma unroll
          for (int k = 0; k < 3; ++k)
#pragma unroll
            for (int b = 0; b < 2; ++b) o[b][c] = mfma16(qf[b], st.part[k], o[b][c]);
        }
      }
#pragma unroll
      for (int c = 0; c < NC; ++c) {
#pragma unroll
        for (int b = 0; b < 2; ++b) o[b][c] *= G[b];
#pragma unroll
        for (int k = 0; k < 3; ++k) {
          o[0][c] = mfma16(p0.part[k], vb[c], o[0][c]);
          o[1][c] = mfma16(p1.part[k], vb[c], o[1][c]);
        }
        const int col = col0 + 16 * c;
        if (col < Vp) {
#pragma unroll
          for (int b = 0; b < 2; ++b) {
            float* op = p.o + ((int64_t)(row0 + t0 + 16 * b + 4 * g4) * H + h) * Vp + col;
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (16 * b + 4 * g4 + r < m) op[(int64_t)r * H * Vp] = o[b][c][r];
          }
        }
      }
    }
    float4v e[2] = {E[0], E[1]};
    float am = a32;
    if (m < 32) {
      am = pw[m];
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 16 * b + 4 * g4 + r;
          e[b][r] = t < m ? pw[max(m - 1 - t, 0)] : 0.f;
        }
    }
    Split vs[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      float4v v[2];
#pragma unroll
      for (int r = 0; r < 8; ++r) v[r >> 2][r & 3] = bf2f((uint16_t)vb[c][r]);
      vs[c] = split8(v[0] * e[0], v[1] * e[1]);
    }
#pragma unroll
    for (int j = 0; j < ND; ++j) {
      // keys transposed: this lane's dimension 16 j + c16 at tokens 4 g4 + r (+ 16)
      const bf16_t* at = B.k + (4 * g4 + (c16 >> 2)) * KS + 16 * j + 4 * (c16 & 3);
      const v4s lo4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s)at);
      const v4s hi4 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4s)(at + 16 * KS));
      const short8 kt = __builtin_shufflevector(lo4, hi4, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
      for (int c = 0; c < NC; ++c) S[j][c] *= am;
#pragma unroll
      for (int k = 0; k < 3; ++k)
#pragma unroll
        for (int c = 0; c < NC; ++c) S[j][c] = mfma16(kt, vs[c].part[k], S[j][c]);
    }
    if (bi + 1 < nblk) lwrite(buf[(bi + 1) & 1], t0 + 32);
  }
  if (slot < 0 || (OUT && !last)) return;
  float* to = OUT ? p.state + ((int64_t)slot * H + h) * Dp * Vp
                  : p.seg + ((int64_t)id * H + h) * Dp * Vp;
#pragma unroll
  for (int j = 0; j < ND; ++j)
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * j + 4 * g4 + r, col = col0 + 16 * c;
        if (d < Dp && col < Vp) to[(int64_t)d * Vp + col] = S[j][c][r];
      }
}

// grid (nseq, H, ceil(Dp * Vp / 1024)): a thread carries 4 state elements over its
// sequence's segments, turning each one's own state into the state it starts from
__global__ __launch_bounds__(256) void chain_kernel(Scan p, int pow_at) {
  const int s = blockIdx.x, h = blockIdx.y;
  const int e = (blockIdx.z * 256 + threadIdx.x) * 4, DV = p.Dp * p.Vp;
  const int all = p.q_start[s + 1] - p.q_start[s], slot = p.slots[s];
  if (all <= p.L || slot < 0 || e >= DV) return;
  const int nseg = (all + p.L - 1) / p.L;
  const float aL = p.pw[h * kPow + pow_at];
  const float4v zero = {0.f, 0.f, 0.f, 0.f};
  float4v S = zero;
  if (p.positions[p.q_start[s]] != 0)
    S = *reinterpret_cast<const float4v*>(p.state + ((int64_t)slot * p.H + h) * DV + e);
  float* seg = p.seg + ((int64_t)seg_base(p.q_start, s, p.L) * p.H + h) * DV + e;
  const int64_t step = (int64_t)p.H * DV;
  for (int j = 0; j < nseg; j += 4) {  // four segments in flight
    float4v own[4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
      own[i] = j + i < nseg - 1 ? *reinterpret_cast<const float4v*>(seg + (j + i) * step) : zero;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (j + i >= nseg) break;
      *reinterpret_cast<float4v*>(seg + (j + i) * step) = S;
      S = S * aL + own[i];
    }
  }
}

// -------------------------------------------------------------- lightning_norm
// one workgroup per row; n = H * Vp columns, 4 a thread and step
template <typename T, int NC>
__global__ __launch_bounds__(256) void norm_kernel(T* __restrict__ y, const float* __restrict__ o,
                                                   Src x, int goff, const float* __restrict__ w,
                                                   int n, float inv_n, float eps) {
  __shared__ float scratch[4];
  const int t = blockIdx.x, tid = threadIdx.x;
  const float4v zero = {0.f, 0.f, 0.f, 0.f};
  float4v v[NC], g[NC];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (tid + 256 * i) * 4;
    v[i] = c < n ? *reinterpret_cast<const float4v*>(o + (int64_t)t * n + c) : zero;
    g[i] = c < n ? x.at4(t, goff + c) : zero;
#pragma unroll
    for (int j = 0; j < 4; ++j) ss += v[i][j] * v[i][j];
  }
  ss = block_sum(ss, scratch);
  const float r = 1.f / sqrtf(ss * inv_n + eps);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (tid + 256 * i) * 4;
    if (c >= n) continue;
    const float4v wv = *reinterpret_cast<const float4v*>(w + c);
    float z[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) z[j] = v[i][j] * r * wv[j] * sigmoidf_(g[i][j]);
    if constexpr (sizeof(T) == 4) {
      *reinterpret_cast<float4v*>(y + (int64_t)t * n + c) = float4v{z[0], z[1], z[2], z[3]};
    } else {
      uint2v k;
      k[0] = pack_bf2(z[0], z[1]);
      k[1] = pack_bf2(z[2], z[3]);
      *reinterpret_cast<uint2v*>(y + (int64_t)t * n + c) = k;
    }
  }
}

bool sizes_ok(int H, int Dp, int Vp) {
  return H >= 1 && H <= 65535 && Dp >= 8 && Dp % 8 == 0 && Vp >= 8 && Vp % 8 == 0 && Dp <= 8192;
}

int any(float* o, float* state, Src x, const float* pw, const int* q_start, int nseq,
        const int* positions, const int* slots, int H, int Dp, int Vp, hipStream_t s) {
  if (nseq > 65535) return -2;
  any_kernel<<<dim3(H, nseq), 256, 2 * Dp * 4, s>>>(o, state, x, pw, q_start, positions, slots, H,
                                                    Dp, Vp);
  return (int)hipGetLastError();
}

int scan(const void* x, int f32, const Scan& p, int n_rows, int pow_at, hipStream_t s) {
  const bool split = n_rows > p.L;  // else every portion is one segment
  const int segs = n_rows / p.L + p.nseq, nc = p.Vp <= 64 || p.Dp > 128 ? 1 : 2;
  const dim3 grid(segs, p.H, (p.Vp + 64 * nc - 1) / (64 * nc));
  const dim3 cgrid(p.nseq, p.H, (p.Dp * p.Vp + 1023) / 1024);
#define OMNIA_LSK(OUT, ND, NC)                                                            \
  do {                                                                                    \
    if (f32) scan_kernel<float, ND, NC, OUT><<<grid, 256, 0, s>>>((const float*)x, p);    \
    else scan16_kernel<ND, NC, OUT><<<grid, 256, 0, s>>>((const bf16_t*)x, p);            \
  } while (0)
#define OMNIA_LS(ND, NC)                                \
  do {                                                  \
    if (split) {                                        \
      OMNIA_LSK(false, ND, NC);                         \
      chain_kernel<<<cgrid, 256, 0, s>>>(p, pow_at);    \
    }                                                   \
    OMNIA_LSK(true, ND, NC);                            \
    return (int)hipGetLastError();                      \
  } while (0)
#define OMNIA_LSD(ND)                   \
  if (p.Dp <= 16 * ND) {                \
    if (nc == 1) OMNIA_LS(ND, 1);       \
    else OMNIA_LS(ND, 2);               \
  }
  OMNIA_LSD(2) OMNIA_LSD(4) OMNIA_LSD(8)
  OMNIA_LS(16, 1);
#undef OMNIA_LSD
#undef OMNIA_LS
#undef OMNIA_LSK
}

// segment length of n_rows rows: enough workgroups to fill the chip, no shorter than 128
int seg_len(int n_rows, int H, int Vp) {
  const int64_t per = (int64_t)H * ((Vp + 127) / 128);
  int L = 128;
  while (L < 4096 && (int64_t)n_rows / (2 * L) * per >= 1024) L *= 2;
  return L;
}

}  // namespace

extern "C" {

int omnia_lightning_pow_cols() { return kPow; }

// fp32 elements of the segment states of a scan
int64_t omnia_lightning_scratch(int n_rows, int nseq, int H, int Dp, int Vp) {
  const int L = seg_len(n_rows, H, Vp);
  return Dp > 256 || n_rows <= L ? 0 : (int64_t)(n_rows / L + nseq) * H * Dp * Vp;
}

// ptype: storage of x -- 0 bf16, 1 fp32, 2 fp16 (slabs); pw [H][kPow]
int omnia_lightning_step(float* o, float* state, const void* x, int ptype, int S, int64_t ld,
                         int64_t slab, const float* pw, const int* positions, const int* slots,
                         int T, int H, int Dp, int Vp, hipStream_t s) {
  if (!sizes_ok(H, Dp, Vp) || S < 1 || ld % 4 || slab % 4) return -1;
  if (T == 0) return 0;
  const Src src{x, ptype, S, ld, slab};
  const int CG = Vp / 4, RG = CG <= 256 ? 256 / CG : 0, nr = RG ? (Dp + RG - 1) / RG : 1 << 20;
  const size_t lds = (size_t)(2 * Dp + Vp + RG * Vp) * 4;
#define OMNIA_ST(N)                                                                           \
  if (nr <= N && lds <= 64 * 1024) {                                                          \
    step_kernel<N><<<dim3(T, H), 256, lds, s>>>(o, state, src, pw, positions, slots, H, Dp,   \
                                                Vp);                                          \
    return (int)hipGetLastError();                                                            \
  }
  OMNIA_ST(1) OMNIA_ST(2) OMNIA_ST(4) OMNIA_ST(8) OMNIA_ST(16) OMNIA_ST(32)
#undef OMNIA_ST
  return any(o, state, src, pw, nullptr, T, positions, slots, H, Dp, Vp, s);
}

int omnia_lightning_scan(float* o, float* state, float* seg, const void* x, int f32, int64_t ldx,
                         const float* pw, const int* q_start, int nseq, const int* positions,
                         const int* slots, int n_rows, int H, int Dp, int Vp, hipStream_t s) {
  if (!sizes_ok(H, Dp, Vp) || ldx % 4 || n_rows < 0) return -1;
  if (nseq == 0 || n_rows == 0) return 0;
  if (Dp > 256)
    return any(o, state, Src{x, f32, 1, ldx, 0}, pw, q_start, nseq, positions, slots, H, Dp, Vp,
               s);
  const int L = seg_len(n_rows, H, Vp);
  int pow_at = kPowSeg;
  while ((64 << (pow_at - kPowSeg)) < L) ++pow_at;
  if (pow_at >= kPow || (n_rows > L && !seg)) return -2;
  const Scan p{o, state, seg, pw, q_start, positions, slots, ldx, nseq, H, Dp, Vp, L};
  return scan(x, f32, p, n_rows, pow_at, s);
}

// w [n] fp32, n = H * Vp; inv_n counts the real columns
int omnia_lightning_norm(void* y, int f32, const float* o, const void* x, int ptype, int S,
                         int64_t ld, int64_t slab, int goff, const float* w, int T, int n,
                         float inv_n, float eps, hipStream_t s) {
  if (n % 4 || n < 4 || n > 16384 || S < 1 || ld % 4 || slab % 4 || goff % 4) return -1;
  if (T == 0) return 0;
  const Src src{x, ptype, S, ld, slab};
#define OMNIA_LN(NC)                                                                         \
  do {                                                                                       \
    if (f32)                                                                                 \
      norm_kernel<float, NC><<<T, 256, 0, s>>>((float*)y, o, src, goff, w, n, inv_n, eps);   \
    else                                                                                     \
      norm_kernel<bf16_t, NC><<<T, 256, 0, s>>>((bf16_t*)y, o, src, goff, w, n, inv_n, eps); \
  } while (0)
  if (n <= 1024) OMNIA_LN(1);
  else if (n <= 2048) OMNIA_LN(2);
  else if (n <= 4096) OMNIA_LN(4);
  else if (n <= 8192) OMNIA_LN(8);
  else OMNIA_LN(16);
#undef OMNIA_LN
  return (int)hipGetLastError();
}

}  // extern "C"
