// Grouped-query attention with a sliding window, query/key norms and attention sinks
// for gfx950: the paged form for any head widths (attention.hip is the 128-wide,
// unlimited one).
//
//   k pages [num_pages][G][page][Dp], v pages [num_pages][G][page][Vp]
//
// Query head h reads key/value head h / (H / G).  A query sees the keys its Mask names (a
// window with kept first keys, a chunk, or all; mask.h); scores may be capped and lose a
// distance bias (score.h); the softmax denominator of head h also holds exp(sink[h]) (sinks
// null: none); a head's output may be multiplied by a gate [T][H].  Scores, softmax, norms
// and gates are fp32.
//
//   gqa_prep     one fused projection row [q (H*Dp) | k (G*Dp) | v (G*Vp)] (or its split-K
//                slabs) -> + bias, per-head RMS norm of q and k, rotary on the first R
//                dimensions (halves or neighbours paired), q rows out (times a factor of
//                their position), k / v rows into the pages; bias, norm, rotation and factor
//                each if asked.  G = 0: q only (a layer that attends to another layer's
//                pages).  Gate columns behind v: their sigmoid, fp32
//   gqa_attend   generic attention (any size, bf16 or fp32), decode and prefill
//   gqa_decode   bf16 decode: Q K^T on MFMA, P V on the VALU, the visible keys cut into
//                equal parts on the device, + gqa_merge
//   gqa_prefill  bf16 prefill (gqa_prefill.hip)
#include "mask.h"
#include "score.h"

using namespace omnia;

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef _Float16 half4v __attribute__((ext_vector_type(4)));

constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float4v mfma16(short8 a, short8 b, float4v c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                 __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

template <typename P>
__device__ __forceinline__ float4v load4(const P* p) {
  if constexpr (sizeof(P) == 4) {
    return *reinterpret_cast<const float4v*>(p);
  } else if constexpr (__is_same(P, _Float16)) {
    const half4v h = *reinterpret_cast<const half4v*>(p);
    return float4v{(float)h[0], (float)h[1], (float)h[2], (float)h[3]};
  } else {
    const short4v h = *reinterpret_cast<const short4v*>(p);
    return float4v{bf2f((uint16_t)h[0]), bf2f((uint16_t)h[1]), bf2f((uint16_t)h[2]),
                   bf2f((uint16_t)h[3])};
  }
}
__device__ __forceinline__ void store4(float* p, float4v v) { *reinterpret_cast<float4v*>(p) = v; }
__device__ __forceinline__ void store4(bf16_t* p, float4v v) {
  uint2v k;
  k[0] = pack_bf2(v[0], v[1]);
  k[1] = pack_bf2(v[2], v[3]);
  *reinterpret_cast<uint2v*>(p) = k;
}

__device__ __forceinline__ int find_seq(const int* q_start, int nseq, int t) {
  int lo = 0, hi = nseq - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (q_start[mid] <= t) lo = mid; else hi = mid - 1;
  }
  return lo;
}

// ------------------------------------------------------------------- gqa_prep
// grid (T, groups of 256 >> lg heads): 1 << lg lanes own one head row of a token, 8
// columns a lane and step (NC steps).
struct PrepArgs {
  const float* wq;
  const float* wk;       // per-dimension norm weights [Dp]; wq null: no norm
  const float* bias;     // per projection column, or null
  const int* positions;
  const int64_t* slots;  // < 0: no write (padded row)
  const float* cos_sin;  // [positions][R] = (cos[R/2] | sin[R/2])
  const float* temp;     // [positions] factors of the queries, or null
  float* gate;           // [T][H], or null
  int64_t ldx, slab;
  int S, H, G, D, Dp, Vp, R, page, lg, pairs;  // pairs: neighbours turn together
  float eps;
};

template <typename T, typename P, int NC>
__global__ __launch_bounds__(256) void prep_kernel(T* __restrict__ q, T* __restrict__ kc,
                                                   T* __restrict__ vc, const P* __restrict__ x,
                                                   PrepArgs a) {
  __shared__ __attribute__((aligned(16))) float rows[256 * NC * 8];
  const int tid = threadIdx.x, lph = 1 << a.lg, l = tid & (lph - 1), t = blockIdx.x;
  const int NH = a.H + 2 * a.G;
  const int hx = blockIdx.y * (256 >> a.lg) + (tid >> a.lg);
  const bool live = hx < NH;
  const int hs = live ? hx : 0;
  const bool isq = hs < a.H, isv = hs >= a.H + a.G;
  const int width = isv ? a.Vp : a.Dp;
  const int col = isv ? (a.H + a.G) * a.Dp + (hs - a.H - a.G) * a.Vp : hs * a.Dp;
  if (a.gate && blockIdx.y == gridDim.y - 1) {
    const P* gr = x + (int64_t)t * a.ldx + (a.H + a.G) * a.Dp + a.G * a.Vp;
    for (int i = tid; i < a.H; i += 256) {
      float z = 0.f;
      for (int s = 0; s < a.S; ++s) z += ldf(gr + s * a.slab + i);
      a.gate[(int64_t)t * a.H + i] = 1.f / (1.f + expf(-z));
    }
  }
  const P* xr = x + (int64_t)t * a.ldx + col;
  const float4v zero = {0.f, 0.f, 0.f, 0.f};
  float4v v[NC][2];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (l + (i << a.lg)) * 8;
    const bool in = c < width;
    v[i][0] = in ? load4(xr + c) : zero;
    v[i][1] = in ? load4(xr + c + 4) : zero;
    for (int s = 1; s < a.S; s += 4) {  // four slabs in flight
      float4v p[4][2];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bool has = in && s + j < a.S;
        p[j][0] = has ? load4(xr + (s + j) * a.slab + c) : zero;
        p[j][1] = has ? load4(xr + (s + j) * a.slab + c + 4) : zero;
      }
#pragma unroll
      for (int e = 0; e < 2; ++e) v[i][e] += (p[0][e] + p[1][e]) + (p[2][e] + p[3][e]);
    }
    if (a.bias && in) {
      v[i][0] += load4(a.bias + col + c);
      v[i][1] += load4(a.bias + col + c + 4);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) ss += v[i][0][j] * v[i][0][j] + v[i][1][j] * v[i][1][j];
  }
  const int pos = a.positions[t], half = a.R >> 1, turned = isv ? 0 : a.R;
  const float* cs = a.cos_sin + (int64_t)pos * a.R;
  const float factor = a.temp && isq ? a.temp[pos] : 1.f;
  float* row = rows + (tid >> a.lg << a.lg) * NC * 8;
  if (!isv && !a.wq) {
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int c = (l + (i << a.lg)) * 8;
      if (c < width) {
        store4(row + c, v[i][0]);
        store4(row + c + 4, v[i][1]);
      }
    }
  } else if (!isv) {
    for (int o = lph >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float r = 1.f / sqrtf(ss / (float)a.D + a.eps);
    const float* w = isq ? a.wq : a.wk;
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int c = (l + (i << a.lg)) * 8;
      if (c < width) {
        v[i][0] = v[i][0] * r * *reinterpret_cast<const float4v*>(w + c);
        v[i][1] = v[i][1] * r * *reinterpret_cast<const float4v*>(w + c + 4);
        store4(row + c, v[i][0]);
        store4(row + c + 4, v[i][1]);
      }
    }
  }
  __syncthreads();
  if (!live) return;
  T* dst;
  if (isq) {
    dst = q + ((int64_t)t * a.H + hs) * a.Dp;
  } else {
    const int64_t slot = a.slots[t];
    if (slot < 0) return;
    const int blk = (int)slot / a.page, off = (int)slot - blk * a.page;
    const int g = isv ? hs - a.H - a.G : hs - a.H;
    dst = (isv ? vc : kc) + (((int64_t)blk * a.G + g) * a.page + off) * width;
  }
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (l + (i << a.lg)) * 8;
    if (c >= width) continue;
    if (c < turned) {
      if (a.pairs) {
#pragma unroll
        for (int e = 0; e < 2; ++e)
#pragma unroll
          for (int j = 0; j < 4; j += 2) {
            const int n = c + 4 * e + j, p = n >> 1;
            if (n < turned) {
              const float x0 = v[i][e][j], x1 = v[i][e][j + 1];
              v[i][e][j] = x0 * cs[p] - x1 * cs[half + p];
              v[i][e][j + 1] = x1 * cs[p] + x0 * cs[half + p];
            }
          }
      } else if ((half & 7) == 0) {  // a chunk lies in one half of the rotated part
        const bool first = c < half;
        const int p = first ? c : c - half;
        const float sg = first ? -1.f : 1.f;
        const float* other = row + (first ? c + half : p);
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float4v cv = *reinterpret_cast<const float4v*>(cs + p + 4 * e);
          const float4v sv = *reinterpret_cast<const float4v*>(cs + half + p + 4 * e);
          const float4v ov = *reinterpret_cast<const float4v*>(other + 4 * e);
#pragma unroll
          for (int j = 0; j < 4; ++j) v[i][e][j] = v[i][e][j] * cv[j] + sg * ov[j] * sv[j];
        }
      } else {
#pragma unroll
        for (int e = 0; e < 2; ++e)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int n = c + 4 * e + j;
            if (n < turned) {
              const bool first = n < half;
              const int p = first ? n : n - half;
              const float other = row[first ? n + half : p];
              v[i][e][j] = v[i][e][j] * cs[p] + (first ? -other : other) * cs[half + p];
            }
          }
      }
    }
    v[i][0] *= factor;
    v[i][1] *= factor;
    if constexpr (sizeof(T) == 4) {
      store4(dst + c, v[i][0]);
      store4(dst + c + 4, v[i][1]);
    } else {
      uint4v k;
      k[0] = pack_bf2(v[i][0][0], v[i][0][1]);
      k[1] = pack_bf2(v[i][0][2], v[i][0][3]);
      k[2] = pack_bf2(v[i][1][0], v[i][1][1]);
      k[3] = pack_bf2(v[i][1][2], v[i][1][3]);
      *reinterpret_cast<uint4v*>(dst + c) = k;
    }
  }
}

// ----------------------------------------------------------------- gqa_attend
// grid (T, H), 256 threads.  Tiles of 256 keys: a thread scores one key, then owns value
// columns.  The sink is the first term of the online softmax.
template <typename T>
__global__ __launch_bounds__(256) void attend_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ kc,
    const T* __restrict__ vc, const int* __restrict__ block_tables, int bt_stride,
    const int* __restrict__ q_start, int nseq, const int* __restrict__ positions, int page, int H,
    int G, int Dp, int Vp, Mask mask, Score score, const float* __restrict__ sinks,
    const float* __restrict__ gate) {
  extern __shared__ float sm[];
  float* qs = sm;        // [Dp]
  float* acc = qs + Dp;  // [Vp]
  float* p = acc + Vp;   // [256]
  float* scratch = p + 256;  // [8]
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, g = h / (H / G);
  const int s = q_start ? find_seq(q_start, nseq, t) : t;
  const int* bt = block_tables + (int64_t)s * bt_stride;
  const int pos = positions[t];
  const int lo = mask.lo(pos), kp = mask.kept(lo), vis = kp + pos + 1 - lo;
  const T* qr = q + ((int64_t)t * H + h) * Dp;
  for (int i = tid; i < Dp; i += 256) qs[i] = ldf(qr + i);
  for (int i = tid; i < Vp; i += 256) acc[i] = 0.f;
  auto at = [&](int i) {  // row in the pages of the i-th visible key
    const int key = i < kp ? i : lo + i - kp;
    return ((int64_t)bt[key / page] * G + g) * page + key % page;
  };
  float m = sinks ? sinks[h] : -INFINITY, l = sinks ? 1.f : 0.f;
  for (int k0 = 0; k0 < vis; k0 += 256) {
    const int n = min(256, vis - k0);
    __syncthreads();
    float sc = -INFINITY;
    if (tid < n) {
      const int i0 = k0 + tid, key = i0 < kp ? i0 : lo + i0 - kp;
      const T* row = kc + at(i0) * Dp;
      float a = 0.f;
      for (int i = 0; i < Dp; ++i) a += qs[i] * ldf(row + i);
      sc = score(a, h, pos - key);
    }
    const float mn = fmaxf(m, block_max(sc, scratch));
    const float e = tid < n ? expf(sc - mn) : 0.f;
    p[tid] = e;
    const float alpha = expf(m - mn);
    l = l * alpha + block_sum(e, scratch);
    m = mn;
    __syncthreads();
    for (int c = tid; c < Vp; c += 256) {
      float a = acc[c] * alpha;
      for (int j = 0; j < n; ++j) a += p[j] * ldf(vc + at(k0 + j) * Vp + c);
      acc[c] = a;
    }
  }
  const float inv = (gate ? gate[(int64_t)t * H + h] : 1.f) / l;
  for (int c = tid; c < Vp; c += 256) stf(out + ((int64_t)t * H + h) * Vp + c, acc[c] * inv);
}

// ----------------------------------------------------------------- gqa_decode
// The visible keys of a row (kept ones, then its window) in parts of part_len keys: decided
// on the device from the live length, so one captured graph splits every context evenly.
constexpr int MIN_PART = 64;

__device__ __forceinline__ int part_len(int n, int splits) {
  return max(((n + splits - 1) / splits + 15) / 16 * 16, MIN_PART);
}

// grid (rows, G * head chunks, splits), NW waves.  KK = Dp / 32; LPR lanes own a value
// row (8 columns each); GH query heads of one key/value head per workgroup (a head past
// the group's end recomputes the last one and is not written).
//   1 scores   each wave takes groups of 16 keys: K rows as the MFMA A operand, Q^T
//              (16 columns, GH real) as B; UG groups of loads in flight
//   2 softmax  per head over the part, in LDS; caps and distance biases here, where every
//              lane has a key
//   3 P V      64 / LPR value rows a wave and step, U steps of loads in flight
template <int KK, int LPR, int GH, int NW>
__global__ __launch_bounds__(64 * NW) void decode_kernel(
    bf16_t* __restrict__ out, float* __restrict__ part_o, float* __restrict__ part_ml,
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ kc, const bf16_t* __restrict__ vc,
    const int* __restrict__ block_tables, int bt_stride, const int* __restrict__ positions, int H,
    int G, int nch, int page_lg, int Vp, Mask mask, Score2 score,
    const float* __restrict__ sinks, const float* __restrict__ gate, int cap) {
  constexpr int Dp = 32 * KK, UG = KK > 4 ? 2 : 4, U = 4, TG = 64 / LPR;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float* stat = reinterpret_cast<float*>(smem);  // [2 * GH], padded to 16
  float* scores = stat + 16;                     // [GH][cap]
  float* red = scores;                           // [NW][GH][Vp]: after the last scores read
  int* pages = reinterpret_cast<int*>(scores + max(GH * cap, NW * GH * Vp));
  const int b = blockIdx.x, g = blockIdx.y / nch, ch0 = blockIdx.y % nch, part = blockIdx.z;
  const int group = H / G, h0 = g * group + ch0 * GH, hn = min(GH, group - ch0 * GH);
  const int pos = positions[b];
  const int lo = mask.lo(pos), kept = mask.kept(lo);
  const int vis = kept + pos + 1 - lo, splits = gridDim.z;
  const int pl = part_len(vis, splits);
  const int p0 = part * pl;
  if (p0 >= vis) return;
  const int n = min(pl, vis - p0), nparts = (vis + pl - 1) / pl;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, pmask = (1 << page_lg) - 1;
  // the part's kept keys p0 .. and, from index nk on, window keys w0 ..; their pages lie
  // behind one another in LDS
  const int nk = max(0, min(kept - p0, n)), w0 = lo + max(0, p0 - kept);
  const int ka = p0 >> page_lg, nkp = nk > 0 ? ((p0 + nk - 1) >> page_lg) - ka + 1 : 0;
  const int wa = w0 >> page_lg;
  const int nwp = n > nk ? ((w0 + n - nk - 1) >> page_lg) - wa + 1 : 0;
  for (int i = tid; i < nkp + nwp; i += 64 * NW)
    pages[i] = block_tables[(int64_t)b * bt_stride + (i < nkp ? ka + i : wa + i - nkp)];

  short8 qf[KK];
  {
    const int c = lane & 15;
    const bf16_t* qrow = q + ((int64_t)b * H + h0 + min(c, hn - 1)) * Dp + 8 * (lane >> 4);
#pragma unroll
    for (int kk = 0; kk < KK; ++kk) qf[kk] = *reinterpret_cast<const short8*>(qrow + 32 * kk);
  }
  __syncthreads();
  auto at = [&](int i) {  // row of the part's i-th key
    const bool k = i < nk;
    const int key = k ? p0 + i : w0 + i - nk;
    return (((int64_t)pages[(key >> page_lg) - (k ? ka : wa - nkp)] * G + g) << page_lg) +
           (key & pmask);
  };
  const int ngroups = (n + 15) / 16;
  for (int grp0 = w; grp0 < ngroups; grp0 += NW * UG) {
    short8 a[UG][KK];
#pragma unroll
    for (int u = 0; u < UG; ++u) {  // groups past the end re-read the last key
      const bf16_t* row = kc + at(min((grp0 + NW * u) * 16 + (lane & 15), n - 1)) * Dp +
                          8 * (lane >> 4);
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) a[u][kk] = *reinterpret_cast<const short8*>(row + 32 * kk);
    }
#pragma unroll
    for (int u = 0; u < UG; ++u) {
      const int grp = grp0 + NW * u;
      if (grp >= ngroups) break;
      float4v acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) acc = mfma16(a[u][kk], qf[kk], acc);
      const int c = lane & 15;  // acc[r]: key grp*16 + 4*(lane>>4) + r, head c
      if (c < GH) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = grp * 16 + 4 * (lane >> 4) + r;
          if (i < n) scores[c * cap + i] = acc[r] * score.mul;
        }
      }
    }
  }
  // first value rows in flight across the softmax
  const int tg = lane / LPR, vch = lane % LPR;
  const bool vlive = vch * 8 < Vp;
  short8 vv[U];
  auto vload = [&](int base) {
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (vlive)
        vv[u] = *reinterpret_cast<const short8*>(
            vc + at(min(base + u * TG * NW + tg, n - 1)) * Vp + vch * 8);
  };
#pragma unroll
  for (int u = 0; u < U; ++u) vv[u] = short8{0, 0, 0, 0, 0, 0, 0, 0};
  vload(w * TG);
  __syncthreads();
  for (int c = w; c < GH; c += NW) {
    float m = -INFINITY;
    if (score.cap > 0.f || score.r1) {
      const int h = h0 + min(c, hn - 1);
      const float r1 = score.r1 ? score.r1[h] : 0.f, r2 = score.r1 ? score.r2[h] : 0.f;
      for (int i = lane; i < n; i += 64) {
        float s = scores[c * cap + i];
        if (score.cap > 0.f) s = score.squash(s);
        const int key = i < nk ? p0 + i : w0 + i - nk;
        s -= r1 * log2_(__builtin_fmaf(r2, (float)(pos - key), 1.f));
        scores[c * cap + i] = s;
        m = fmaxf(m, s);
      }
    } else {
      for (int i = lane; i < n; i += 64) m = fmaxf(m, scores[c * cap + i]);
    }
    m = wave_max(m);
    float s = 0.f;
    for (int i = lane; i < n; i += 64) {
      const float p = exp2f(scores[c * cap + i] - m);
      scores[c * cap + i] = p;
      s += p;
    }
    s = wave_sum(s);
    if (lane == 0) {
      stat[2 * c] = m;
      stat[2 * c + 1] = s;
    }
  }
  __syncthreads();
  float acc[GH][8];
#pragma unroll
  for (int c = 0; c < GH; ++c)
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[c][j] = 0.f;
  for (int base = w * TG; base < n; base += TG * NW * U) {
    short8 cur[U];
#pragma unroll
    for (int u = 0; u < U; ++u) cur[u] = vv[u];
    vload(base + TG * NW * U);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int i = base + u * TG * NW + tg;
      if (i < n) {
#pragma unroll
        for (int c = 0; c < GH; ++c) {
          const float p = scores[c * cap + i];
#pragma unroll
          for (int j = 0; j < 8; ++j) acc[c][j] += p * bf2f((uint16_t)cur[u][j]);
        }
      }
    }
  }
#pragma unroll
  for (int c = 0; c < GH; ++c)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      float v = acc[c][j];
#pragma unroll
      for (int o = LPR; o < 64; o <<= 1) v += __shfl_xor(v, o, 64);
      acc[c][j] = v;
    }
  __syncthreads();  // every wave is done with `scores`, which `red` overlays
  if (tg == 0 && vlive) {
#pragma unroll
    for (int c = 0; c < GH; ++c)
#pragma unroll
      for (int j = 0; j < 8; ++j) red[(w * GH + c) * Vp + vch * 8 + j] = acc[c][j];
  }
  __syncthreads();
  for (int i = tid; i < hn * Vp; i += 64 * NW) {
    const int c = i / Vp, d = i - c * Vp, h = h0 + c;
    float v = 0.f;
#pragma unroll
    for (int k = 0; k < NW; ++k) v += red[(k * GH + c) * Vp + d];
    const float m = stat[2 * c], s = stat[2 * c + 1];
    if (nparts == 1) {
      if (sinks) {
        const float sk = sinks[h] * kLog2e, mm = fmaxf(m, sk), e = exp2f(m - mm);
        v = v * e / (s * e + exp2f(sk - mm));
      } else {
        v = v / s;
      }
      if (gate) v *= gate[(int64_t)b * H + h];
      out[((int64_t)b * H + h) * Vp + d] = f2bf(v);
    } else {
      const int64_t slot = ((int64_t)b * H + h) * splits + part;
      part_o[slot * Vp + d] = v;
      if (d == 0) {
        part_ml[slot * 2] = m;
        part_ml[slot * 2 + 1] = s;
      }
    }
  }
}

// grid (rows * H), 128 threads
__global__ __launch_bounds__(128) void merge_kernel(bf16_t* __restrict__ out,
                                                    const float* __restrict__ part_o,
                                                    const float* __restrict__ part_ml,
                                                    const int* __restrict__ positions, int H,
                                                    int Vp, Mask mask, int splits,
                                                    const float* __restrict__ sinks,
                                                    const float* __restrict__ gate) {
  extern __shared__ float wt[];  // [splits]
  __shared__ float scratch[2];
  const int bh = blockIdx.x, b = bh / H, h = bh - b * H;
  const int pos = positions[b];
  const int lo = mask.lo(pos), vis = mask.kept(lo) + pos + 1 - lo;
  const int pl = part_len(vis, splits), nparts = (vis + pl - 1) / pl;
  if (nparts <= 1) return;
  const float* ml = part_ml + (int64_t)bh * splits * 2;
  const float* po = part_o + (int64_t)bh * splits * Vp;
  const int tid = threadIdx.x;
  const float sk = sinks ? sinks[h] * kLog2e : -INFINITY;
  float m = sk;
  for (int p = tid; p < nparts; p += 128) m = fmaxf(m, ml[2 * p]);
  m = block_max(m, scratch);
  float tot = 0.f;
  for (int p = tid; p < nparts; p += 128) {
    wt[p] = exp2f(ml[2 * p] - m);
    tot += wt[p] * ml[2 * p + 1];
  }
  tot = block_sum(tot, scratch) + (sinks ? exp2f(sk - m) : 0.f);  // (orders wt as well)
  const float inv = (gate ? gate[bh] : 1.f) / tot;
  for (int d = tid; d < Vp; d += 128) {
    float v = 0.f;
    for (int p = 0; p < nparts; p += 8) {  // eight parts in flight
      float x[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) x[k] = po[(int64_t)min(p + k, nparts - 1) * Vp + d];
#pragma unroll
      for (int k = 0; k < 8; ++k) v += p + k < nparts ? wt[min(p + k, nparts - 1)] * x[k] : 0.f;
    }
    out[(int64_t)bh * Vp + d] = f2bf(v * inv);
  }
}

int log2i(int n) {
  for (int i = 0; i < 31; ++i)
    if (n == (1 << i)) return i;
  return -1;
}

}  // namespace

extern "C" {

// ptype: storage of x -- 0 bf16, 1 fp32, 2 fp16 (slabs)
int omnia_gqa_prep(void* q, void* kc, void* vc, int f32, const void* x, int ptype, int S,
                   int64_t slab, int64_t ldx, const float* wq, const float* wk,
                   const float* bias, const int* positions, const int64_t* slots,
                   const float* cos_sin, int pairs, int T, int H, int G, int D, int Dp, int Vp,
                   int R, int page, float eps, const float* temp, float* gate, hipStream_t s) {
  if (Dp % 8 || Vp % 8 || ldx % 8 || slab % 8 || S < 1 || R % 2 || R > D || D > Dp || page < 1)
    return -1;
  const int w = Dp > Vp || G == 0 ? Dp : Vp;
  if (w > 1024) return -2;
  if (T == 0) return 0;
  int lg = 2;
  while (lg < 6 && (8 << lg) < w) ++lg;
  const PrepArgs a{wq, wk, bias, positions, slots, cos_sin, temp, gate, ldx, slab, S,
                   H,  G,  D,    Dp,        Vp,    R,       page, lg,  pairs, eps};
  const int hpb = 256 >> lg;
  const dim3 grid(T, (H + 2 * G + hpb - 1) / hpb);
#define OMNIA_GP(TT, PP)                                                                       \
  do {                                                                                         \
    if (w <= 512)                                                                              \
      prep_kernel<TT, PP, 1><<<grid, 256, 0, s>>>((TT*)q, (TT*)kc, (TT*)vc, (const PP*)x, a);  \
    else                                                                                       \
      prep_kernel<TT, PP, 2><<<grid, 256, 0, s>>>((TT*)q, (TT*)kc, (TT*)vc, (const PP*)x, a);  \
  } while (0)
  if (f32) {
    if (ptype != 1) return -3;
    OMNIA_GP(float, float);
  } else if (ptype == 0) {
    OMNIA_GP(bf16_t, bf16_t);
  } else if (ptype == 1) {
    OMNIA_GP(bf16_t, float);
  } else {
    OMNIA_GP(bf16_t, _Float16);
  }
#undef OMNIA_GP
  return (int)hipGetLastError();
}

int omnia_gqa_attend(void* out, int f32, const void* q, const void* kc, const void* vc,
                     const int* block_tables, int bt_stride, const int* q_start, int nseq,
                     const int* positions, int T, int page, int H, int G, int Dp, int Vp,
                     Mask mask, Score score, const float* sinks, const float* gate,
                     hipStream_t s) {
  if (G < 1 || H % G || page < 1 || !mask.ok() || !score.ok()) return -1;
  if (T == 0) return 0;
  const size_t lds = (size_t)(Dp + Vp + 256 + 8) * 4;
  if (lds > 64 * 1024 || H > 65535) return -2;
  const dim3 grid(T, H);
  if (f32)
    attend_kernel<float><<<grid, 256, lds, s>>>((float*)out, (const float*)q, (const float*)kc,
                                                (const float*)vc, block_tables, bt_stride, q_start,
                                                nseq, positions, page, H, G, Dp, Vp, mask, score,
                                                sinks, gate);
  else
    attend_kernel<bf16_t><<<grid, 256, lds, s>>>(
        (bf16_t*)out, (const bf16_t*)q, (const bf16_t*)kc, (const bf16_t*)vc, block_tables,
        bt_stride, q_start, nseq, positions, page, H, G, Dp, Vp, mask, score, sinks, gate);
  return (int)hipGetLastError();
}

// max_ctx: no context is longer than this (sizes the score tile)
int omnia_gqa_decode(void* out, float* part_o, float* part_ml, const void* q, const void* kc,
                     const void* vc, const int* block_tables, int bt_stride, const int* positions,
                     int T, int page, int H, int G, int Dp, int Vp, Mask mask, Score score,
                     const float* sinks, const float* gate, int splits, int max_ctx,
                     hipStream_t s) {
  const int max_keys = mask.ok() ? mask.most(max_ctx) : 0;
  const int lg = log2i(page);
  if (lg < 0 || G < 1 || H % G || Dp % 32 || Dp > 256 || Vp % 8 || Vp > 256 || splits < 1 ||
      max_keys < 1 || H > 65535 || splits > 8192 || !score.ok())
    return -1;
  if (T == 0) return 0;
  const int group = H / G, gh = group >= 5 ? 8 : group >= 3 ? 4 : group;
  const int nch = (group + gh - 1) / gh;
  int cap = ((max_keys + splits - 1) / splits + 15) / 16 * 16;
  cap = cap < MIN_PART ? MIN_PART : cap;
  // two-wave workgroups once there are enough of them to keep the chip's loads in flight
  const int nw = (int64_t)T * G * nch * splits >= 1024 ? 2 : 4;
  const int tile = gh * cap > nw * gh * Vp ? gh * cap : nw * gh * Vp;
  const size_t lds = 64 + (size_t)tile * 4 + (size_t)(cap / page + 4) * 4;
  if (lds > 96 * 1024) return -2;
  const dim3 grid(T, G * nch, splits);
  const Score2 sc(score);
#define OMNIA_GD(KK, LP, GH, NN)                                                               \
  decode_kernel<KK, LP, GH, NN><<<grid, 64 * NN, lds, s>>>(                                    \
      (bf16_t*)out, part_o, part_ml, (const bf16_t*)q, (const bf16_t*)kc, (const bf16_t*)vc,   \
      block_tables, bt_stride, positions, H, G, nch, lg, Vp, mask, sc, sinks, gate, cap)
#define OMNIA_GD_N(KK, LP, GH) \
  do { if (nw == 2) OMNIA_GD(KK, LP, GH, 2); else OMNIA_GD(KK, LP, GH, 4); } while (0)
#define OMNIA_GD_G(KK, LP)                      \
  do {                                          \
    if (gh == 1) OMNIA_GD_N(KK, LP, 1);         \
    else if (gh == 2) OMNIA_GD_N(KK, LP, 2);    \
    else if (gh == 4) OMNIA_GD_N(KK, LP, 4);    \
    else OMNIA_GD_N(KK, LP, 8);                 \
  } while (0)
#define OMNIA_GD_K(KK)                          \
  case KK:                                      \
    if (Vp <= 64) OMNIA_GD_G(KK, 8);            \
    else if (Vp <= 128) OMNIA_GD_G(KK, 16);     \
    else OMNIA_GD_G(KK, 32);                    \
    break
  switch (Dp / 32) {
    OMNIA_GD_K(1);
    OMNIA_GD_K(2);
    OMNIA_GD_K(3);
    OMNIA_GD_K(4);
    OMNIA_GD_K(6);
    OMNIA_GD_K(8);
    default: return -3;
  }
#undef OMNIA_GD_K
#undef OMNIA_GD_G
#undef OMNIA_GD_N
#undef OMNIA_GD
  if (splits > 1)
    merge_kernel<<<T * H, 128, splits * 4, s>>>((bf16_t*)out, part_o, part_ml, positions, H, Vp, mask,
                                       splits, sinks, gate);
  return (int)hipGetLastError();
}

}  // extern "C"
