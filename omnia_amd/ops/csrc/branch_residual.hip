// Residual step behind a layer with two output projections side by side (bf16 or fp32
// models, fp32 residual):
//
//     x += rms(a) * wa + rms(b) * wb ;  h = x, or the next sublayer's norm of x
//
// a and b: projections (bf16 / fp32) or their split-K slabs (fp32 / fp16), each with a
// bias if given; rms statistics over the inv_n real columns (padding columns hold zeros
// and have zero weights; a constant on a branch is part of its weight).  The next norm is
// Dynamic Tanh, tanh(alpha x) w + b, or an RMS norm.
//
// One workgroup per row; a thread keeps its columns of both branches in registers between
// the statistics and the update.
#include "common.h"

using namespace omnia;

namespace {

typedef _Float16 half4v __attribute__((ext_vector_type(4)));

struct Branch {
  const void* m;
  int type, S;  // storage 0 bf16, 1 fp32, 2 fp16; slabs
  int64_t row, slab;
  const float* bias;  // or null
  const float* w;
};
struct Next {  // w null: identity; b null: RMS, else tanh
  float alpha;
  const float* w;
  const float* b;
};

// PT: the storage type if both branches have it, else -1 (looked up: slower, since every
// load is then waited for in its own branch)
template <int PT>
__device__ __forceinline__ float4v load4(const void* base, int type, int64_t at) {
  if constexpr (PT >= 0) type = PT;
  if (type == 1) return *reinterpret_cast<const float4v*>((const float*)base + at);
  if (type == 2) {
    const half4v h = *reinterpret_cast<const half4v*>((const _Float16*)base + at);
    return float4v{(float)h[0], (float)h[1], (float)h[2], (float)h[3]};
  }
  const short4v h = *reinterpret_cast<const short4v*>((const bf16_t*)base + at);
  return float4v{bf2f((uint16_t)h[0]), bf2f((uint16_t)h[1]), bf2f((uint16_t)h[2]),
                 bf2f((uint16_t)h[3])};
}
__device__ __forceinline__ void store4(float* p, float4v v) { *reinterpret_cast<float4v*>(p) = v; }
__device__ __forceinline__ void store4(bf16_t* p, float4v v) {
  uint2v k;
  k[0] = pack_bf2(v[0], v[1]);
  k[1] = pack_bf2(v[2], v[3]);
  *reinterpret_cast<uint2v*>(p) = k;
}

// columns of a thread: c = (threadIdx.x + i * NT) * 4, i < NC
template <typename T, int PT, int NT, int NC>
__global__ __launch_bounds__(NT) void branch_kernel(T* __restrict__ h, float* __restrict__ x,
                                                    int d, Branch ba, Branch bb, float inv_n,
                                                    float eps, Next next) {
  __shared__ float red[2][NT / 64];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x;
  const float4v zero = {0.f, 0.f, 0.f, 0.f};
  float4v a[NC], b[NC], old[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (tid + i * NT) * 4;
    const bool in = c < d;
    a[i] = in ? load4<PT>(ba.m, ba.type, t * ba.row + c) : zero;
    b[i] = in ? load4<PT>(bb.m, bb.type, t * bb.row + c) : zero;
    old[i] = in ? *reinterpret_cast<const float4v*>(x + t * d + c) : zero;
  }
  auto slabs = [&](float4v (&v)[NC], const Branch& p) {
    for (int s = 1; s < p.S; s += 4) {  // four slabs in flight
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        const int c = (tid + i * NT) * 4;
        if (c < d) {
          float4v q[4];
#pragma unroll
          for (int j = 0; j < 4; ++j)
            q[j] = s + j < p.S ? load4<PT>(p.m, p.type, (s + j) * p.slab + t * p.row + c) : zero;
          v[i] += (q[0] + q[1]) + (q[2] + q[3]);
        }
      }
    }
    if (p.bias) {
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        const int c = (tid + i * NT) * 4;
        if (c < d) v[i] += *reinterpret_cast<const float4v*>(p.bias + c);
      }
    }
  };
  slabs(a, ba);
  slabs(b, bb);
  float sa = 0.f, sb = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      sa += a[i][j] * a[i][j];
      sb += b[i][j] * b[i][j];
    }
  sa = wave_sum(sa);
  sb = wave_sum(sb);
  if ((tid & 63) == 0) {
    red[0][tid >> 6] = sa;
    red[1][tid >> 6] = sb;
  }
  __syncthreads();
  sa = sb = 0.f;
#pragma unroll
  for (int k = 0; k < NT / 64; ++k) {
    sa += red[0][k];
    sb += red[1][k];
  }
  const float ra = 1.f / sqrtf(sa * inv_n + eps), rb = 1.f / sqrtf(sb * inv_n + eps);
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (tid + i * NT) * 4;
    if (c < d) {
      const float4v wa = *reinterpret_cast<const float4v*>(ba.w + c);
      const float4v wb = *reinterpret_cast<const float4v*>(bb.w + c);
      old[i] += a[i] * ra * wa + b[i] * rb * wb;
      store4(x + t * d + c, old[i]);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) ss += old[i][j] * old[i][j];
  }
  float r = 1.f;
  if (next.w && !next.b) {  // RMS
    ss = wave_sum(ss);
    __syncthreads();
    if ((tid & 63) == 0) red[0][tid >> 6] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int k = 0; k < NT / 64; ++k) ss += red[0][k];
    r = 1.f / sqrtf(ss * inv_n + eps);
  }
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (tid + i * NT) * 4;
    if (c >= d) continue;
    float4v v = old[i];
    if (next.w) {
      const float4v w = *reinterpret_cast<const float4v*>(next.w + c);
      if (next.b) {
        const float4v bv = *reinterpret_cast<const float4v*>(next.b + c);
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = tanhf(next.alpha * v[j]) * w[j] + bv[j];
      } else {
        v = v * r * w;
      }
    }
    store4(h + t * d + c, v);
  }
}

}  // namespace

extern "C" int omnia_branch_residual(void* h, int f32, float* x, int rows, int d, const void* a,
                                     int at, int aS, int64_t arow, int64_t aslab,
                                     const float* abias, const float* aw, const void* b, int bt,
                                     int bS, int64_t brow, int64_t bslab, const float* bbias,
                                     const float* bw, float inv_n, float eps, float alpha,
                                     const float* nw, const float* nb, hipStream_t s) {
  if (d % 4 || d < 4 || d > 16384 || aS < 1 || bS < 1 || arow % 4 || aslab % 4 || brow % 4 ||
      bslab % 4 || !aw || !bw || (f32 && (at != 1 || bt != 1)))
    return -1;
  if (rows == 0) return 0;
  const Branch ba{a, at, aS, arow, aslab, abias, aw}, bb{b, bt, bS, brow, bslab, bbias, bw};
  const Next next{alpha, nw, nb};
#define OMNIA_BRP(TT, PT, NT, NC) \
  branch_kernel<TT, PT, NT, NC><<<rows, NT, 0, s>>>((TT*)h, x, d, ba, bb, inv_n, eps, next)
#define OMNIA_BR(NT, NC)                                        \
  do {                                                          \
    if (f32) OMNIA_BRP(float, 1, NT, NC);                       \
    else if (at != bt) OMNIA_BRP(bf16_t, -1, NT, NC);           \
    else if (at == 0) OMNIA_BRP(bf16_t, 0, NT, NC);             \
    else if (at == 1) OMNIA_BRP(bf16_t, 1, NT, NC);             \
    else OMNIA_BRP(bf16_t, 2, NT, NC);                          \
  } while (0)
  if (d <= 1024) OMNIA_BR(256, 1);
  else if (rows <= 512 && d <= 4096) OMNIA_BR(1024, 1);
  else if (d <= 2048) OMNIA_BR(256, 2);
  else if (d <= 4096) OMNIA_BR(512, 2);
  else if (d <= 8192) OMNIA_BR(1024, 2);
  else OMNIA_BR(1024, 4);
#undef OMNIA_BR
#undef OMNIA_BRP
  return (int)hipGetLastError();
}
