// Dynamic-Tanh normalisation, fused with what surrounds it (bf16 or fp32 models):
//
//     norm(x) = tanh(alpha * x) * w + b          (no statistics over the row)
//
//   tanh_norm_embed      token embedding gather -> fp32 residual row, and the first
//                        layer's normed input
//   tanh_norm_residual   x += norm1(m + bias); h = norm2(x): the residual update after
//                        a sublayer and the next sublayer's input in one pass (norm1: or
//                        none).  `m` is a projection's bf16 / fp32 output, its S split-K
//                        slabs or S parts per row (the slots of a token's experts, where
//                        an identity expert's slot stands for its weight times the
//                        sublayer's input and holds nothing)
//   glu                  act(g + bg) * (u + bu) of a [gate | up] projection (same inputs
//                        as above), act = silu or the tanh form of gelu; biases if given
//
// The residual stream is fp32.  All are memory-bound; because the norm has no
// reduction there is no row ownership: threads cover the flat [rows, d] matrix,
// 4 columns each.
#include "common.h"

using namespace omnia;

namespace {

typedef _Float16 half4v __attribute__((ext_vector_type(4)));

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

// one element of a projection given as S slabs of `slab` elements
template <typename P>
__device__ __forceinline__ float4v sum_slabs(const P* p, int S, int64_t slab) {
  float4v a = load4(p);
  for (int s = 1; s < S; ++s) a += load4(p + s * slab);
  return a;
}

__device__ __forceinline__ float4v norm4(float4v x, float alpha, const float* w, const float* b) {
  const float4v wv = *reinterpret_cast<const float4v*>(w);
  const float4v bv = *reinterpret_cast<const float4v*>(b);
  float4v y;
#pragma unroll
  for (int j = 0; j < 4; ++j) y[j] = tanhf(alpha * x[j]) * wv[j] + bv[j];
  return y;
}

struct Post {  // norm of the sublayer's output; w null: none
  float alpha;
  const float* w;
  const float* b;
};
// identity experts among the parts of a row: those with ids >= first
template <typename T>
struct Identity {
  const int* ids;  // [rows, S]; null: none
  const float* wts;
  const T* in;  // [rows, d]
  int first;
};

template <typename T>
__global__ __launch_bounds__(256) void embed_kernel(
    T* __restrict__ h, float* __restrict__ x, const int* __restrict__ ids,
    const T* __restrict__ table, int d, int vocab, float alpha, const float* __restrict__ w,
    const float* __restrict__ b, const int64_t* __restrict__ src,
    const int* __restrict__ tok_slots) {
  const int t = blockIdx.x;
  const int64_t sl = src ? src[t] : -1;
  const int id = sl >= 0 ? tok_slots[sl] : ids[t];
  const bool ok = id >= 0 && id < vocab;
  const T* row = table + (int64_t)(ok ? id : 0) * d;
  for (int c = threadIdx.x * 4; c < d; c += 1024) {
    const float4v v = ok ? load4(row + c) : float4v{0.f, 0.f, 0.f, 0.f};
    store4(x + (int64_t)t * d + c, v);
    store4(h + (int64_t)t * d + c, norm4(v, alpha, w + c, b + c));
  }
}

template <typename T, typename P>
__global__ __launch_bounds__(256) void residual_kernel(
    T* __restrict__ h, float* __restrict__ x, const P* __restrict__ m, int S, int64_t row,
    int64_t slab, int d, const float* __restrict__ bias, Post post, Identity<T> idn, float a2,
    const float* __restrict__ w2, const float* __restrict__ b2) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (c >= d) return;
  const int64_t e = (int64_t)blockIdx.y * d + c;
  const P* mr = m + blockIdx.y * row + c;
  float4v v;
  if (idn.ids) {
    const float4v hv = load4(idn.in + e);
    const int* ids = idn.ids + (int64_t)blockIdx.y * S;
    const float* wts = idn.wts + (int64_t)blockIdx.y * S;
    v = float4v{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < S; ++s) v += ids[s] < idn.first ? load4(mr + s * slab) : hv * wts[s];
  } else {
    v = sum_slabs(mr, S, slab);
  }
  if (bias) v += *reinterpret_cast<const float4v*>(bias + c);
  if (post.w) v = norm4(v, post.alpha, post.w + c, post.b + c);
  const float4v r = *reinterpret_cast<const float4v*>(x + e) + v;
  store4(x + e, r);
  store4(h + e, norm4(r, a2, w2 + c, b2 + c));
}

template <typename T, typename P, int ACT>
__global__ __launch_bounds__(256) void glu_kernel(T* __restrict__ out, const P* __restrict__ m,
                                                  int S, int64_t slab, int inter,
                                                  const float* __restrict__ bias) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (c >= inter) return;
  const P* row = m + (int64_t)blockIdx.y * 2 * inter;
  float4v g = sum_slabs(row + c, S, slab), u = sum_slabs(row + inter + c, S, slab);
  if (bias) {
    g += *reinterpret_cast<const float4v*>(bias + c);
    u += *reinterpret_cast<const float4v*>(bias + inter + c);
  }
  float4v o;
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = (ACT ? gelu_tanh_(g[j]) : siluf_(g[j])) * u[j];
  store4(out + (int64_t)blockIdx.y * inter + c, o);
}

}  // namespace

extern "C" {

// ptype: storage of `m` -- 0 bf16, 1 fp32, 2 fp16 (slabs)
int omnia_tanh_norm_embed(void* h, float* x, const int* ids, const void* table, int f32, int T,
                          int d, int vocab, float alpha, const float* w, const float* b,
                          const int64_t* src, const int* tok_slots, hipStream_t s) {
  if (d % 4 || d < 4) return -1;
  if (src && !tok_slots) return -2;
  if (T == 0) return 0;
  if (f32)
    embed_kernel<float><<<T, 256, 0, s>>>((float*)h, x, ids, (const float*)table, d, vocab, alpha,
                                          w, b, src, tok_slots);
  else
    embed_kernel<bf16_t><<<T, 256, 0, s>>>((bf16_t*)h, x, ids, (const bf16_t*)table, d, vocab,
                                           alpha, w, b, src, tok_slots);
  return (int)hipGetLastError();
}

int omnia_tanh_norm_residual(void* h, int f32, float* x, const void* m, int ptype, int S,
                             int64_t row, int64_t slab, int rows, int d, const float* bias,
                             float a1, const float* w1, const float* b1, float a2,
                             const float* w2, const float* b2, const int* ids, const float* wts,
                             const void* in, int first, hipStream_t s) {
  if (ids && (!wts || !in)) return -3;
  if (d % 4 || d < 4 || S < 1 || row % 4 || slab % 4 || rows > 65535) return -1;
  if (rows == 0) return 0;
  const dim3 grid((d / 4 + 255) / 256, rows);
#define OMNIA_TNR(T, P)                                                                      \
  residual_kernel<T, P><<<grid, 256, 0, s>>>((T*)h, x, (const P*)m, S, row, slab, d, bias,     \
                                             Post{a1, w1, b1},                                 \
                                             Identity<T>{ids, wts, (const T*)in, first}, a2,   \
                                             w2, b2)
  if (f32) {
    if (ptype != 1) return -2;
    OMNIA_TNR(float, float);
  } else if (ptype == 0) {
    OMNIA_TNR(bf16_t, bf16_t);
  } else if (ptype == 1) {
    OMNIA_TNR(bf16_t, float);
  } else {
    OMNIA_TNR(bf16_t, _Float16);
  }
#undef OMNIA_TNR
  return (int)hipGetLastError();
}

int omnia_glu(void* out, int f32, const void* m, int ptype, int S, int rows, int inter,
              const float* bias, int gelu, hipStream_t s) {
  if (inter % 4 || inter < 4 || S < 1 || rows > 65535) return -1;
  if (rows == 0) return 0;
  const dim3 grid((inter / 4 + 255) / 256, rows);
  const int64_t slab = (int64_t)rows * 2 * inter;
#define OMNIA_GLU_A(T, P, A) \
  glu_kernel<T, P, A><<<grid, 256, 0, s>>>((T*)out, (const P*)m, S, slab, inter, bias)
#define OMNIA_GLU(T, P)                                           \
  do {                                                            \
    if (gelu) OMNIA_GLU_A(T, P, 1);                               \
    else OMNIA_GLU_A(T, P, 0);                                    \
  } while (0)
  if (f32) {
    if (ptype != 1) return -2;
    OMNIA_GLU(float, float);
  } else if (ptype == 0) {
    OMNIA_GLU(bf16_t, bf16_t);
  } else if (ptype == 1) {
    OMNIA_GLU(bf16_t, float);
  } else {
    OMNIA_GLU(bf16_t, _Float16);
  }
#undef OMNIA_GLU
#undef OMNIA_GLU_A
  return (int)hipGetLastError();
}

}  // extern "C"
