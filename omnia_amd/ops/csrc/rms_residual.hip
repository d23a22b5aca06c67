// RMS norms around an fp32 residual stream, fused with what surrounds them (bf16 or fp32
// models).  A norm is x / sqrt(sum(x^2) * inv_n + eps) * w with fp32 weights w (a weight
// stored around zero arrives here as 1 + w); inv_n counts the real columns, padding
// columns hold zeros and have w = 0.
//
//   rms_embed     token embedding gather [-> norm] -> fp32 residual row, and the first
//                 sublayer's input (the residual itself, or its pre-norm)
//   rms_residual  x += norm(sum of m's parts + bias); h = x or pre-norm(x): what follows a
//                 sublayer, in one pass.  Parts: split-K slabs of a projection, or the
//                 slots of a token's experts
//   softcap       logits <- cap * tanh(logits / cap), in place
//
// One workgroup per row; a thread keeps its columns in registers between the statistic
// and the update.  Few rows (decode): 1024 threads a row, so that a row's loads are all
// in flight at once.
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

struct Norm {
  const float* w;  // null: identity
  float inv_n, eps;
};

// columns of a thread: c = (threadIdx.x + i * NT) * 4, i < NC
template <int NT, int NC>
__device__ __forceinline__ void norm_row(float4v (&v)[NC], int d, Norm n, float* scratch) {
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) ss += v[i][j] * v[i][j];
  ss = block_sum(ss, scratch);
  const float r = 1.f / sqrtf(ss * n.inv_n + n.eps);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    if (c < d) v[i] = v[i] * r * *reinterpret_cast<const float4v*>(n.w + c);
  }
}

template <typename T, int NT, int NC>
__global__ __launch_bounds__(NT) void embed_kernel(T* __restrict__ h, float* __restrict__ x,
                                                    const int* __restrict__ ids,
                                                    const T* __restrict__ table, int d, int vocab,
                                                    Norm emb, Norm pre,
                                                    const int64_t* __restrict__ src,
                                                    const int* __restrict__ tok_slots) {
  __shared__ float scratch[NT / 64];
  const int t = blockIdx.x;
  const int64_t sl = src ? src[t] : -1;
  const int id = sl >= 0 ? tok_slots[sl] : ids[t];
  const bool ok = id >= 0 && id < vocab;
  const T* row = table + (int64_t)(ok ? id : 0) * d;
  float4v v[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    v[i] = float4v{0.f, 0.f, 0.f, 0.f};
    if (ok && c < d) v[i] = load4(row + c);
  }
  if (emb.w) norm_row<NT, NC>(v, d, emb, scratch);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    if (c < d) store4(x + (int64_t)t * d + c, v[i]);
  }
  if (pre.w) norm_row<NT, NC>(v, d, pre, scratch);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    if (c < d) store4(h + (int64_t)t * d + c, v[i]);
  }
}

template <typename T, typename P, int NT, int NC>
__global__ __launch_bounds__(NT) void residual_kernel(T* __restrict__ h, float* __restrict__ x,
                                                       const P* __restrict__ m, int S,
                                                       int64_t row_stride, int64_t part_stride,
                                                       int d, const float* __restrict__ bias,
                                                       Norm post, Norm pre) {
  __shared__ float scratch[NT / 64];
  const int64_t t = blockIdx.x;
  const P* mr = m + t * row_stride;
  float* xr = x + t * d;
  const float4v zero = {0.f, 0.f, 0.f, 0.f};
  float4v v[NC], old[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    v[i] = c < d ? load4(mr + c) : zero;
    old[i] = c < d ? *reinterpret_cast<const float4v*>(xr + c) : zero;
    if (bias && c < d) v[i] += *reinterpret_cast<const float4v*>(bias + c);
  }
  for (int s = 1; s < S; s += 4) {  // four parts in flight
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int c = (threadIdx.x + i * NT) * 4;
      if (c < d) {
        float4v p[4];
#pragma unroll
        for (int j = 0; j < 4; ++j)
          p[j] = s + j < S ? load4(mr + (s + j) * part_stride + c) : zero;
        v[i] += (p[0] + p[1]) + (p[2] + p[3]);
      }
    }
  }
  norm_row<NT, NC>(v, d, post, scratch);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    if (c < d) {
      v[i] += old[i];
      store4(xr + c, v[i]);
    }
  }
  if (pre.w) norm_row<NT, NC>(v, d, pre, scratch);
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int c = (threadIdx.x + i * NT) * 4;
    if (c < d) store4(h + t * d + c, v[i]);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(T* __restrict__ z, int64_t n, float cap,
                                                      float inv) {
  const int64_t stride = (int64_t)gridDim.x * 256;
  const int64_t n4 = n / 4, i0 = (int64_t)blockIdx.x * 256 + threadIdx.x;
  for (int64_t i = i0; i < n4; i += stride) {
    float4v v = load4(z + 4 * i);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = cap * tanhf(v[j] * inv);
    store4(z + 4 * i, v);
  }
  const int64_t e = 4 * n4 + i0;
  if (e < n) stf(z + e, cap * tanhf(ldf(z + e) * inv));
}

}  // namespace

// (threads, chunks of 4 columns a thread) of a row
#define OMNIA_NC(K)                                 \
  do {                                              \
    if (d <= 1024) K(256, 1);                       \
    else if (rows <= 512 && d <= 4096) K(1024, 1);  \
    else if (rows <= 512 && d <= 8192) K(1024, 2);  \
    else if (rows <= 512) K(1024, 4);               \
    else if (d <= 2048) K(256, 2);                  \
    else if (d <= 4096) K(256, 4);                  \
    else if (d <= 8192) K(256, 8);                  \
    else K(256, 16);                                \
  } while (0)

extern "C" {

int omnia_rms_embed(void* h, float* x, const int* ids, const void* table, int f32, int T, int d,
                    int vocab, const float* we, const float* wp, float inv_n, float eps,
                    const int64_t* src, const int* tok_slots, hipStream_t s) {
  if (d % 4 || d < 4 || d > 16384) return -1;
  if (src && !tok_slots) return -2;
  if (T == 0) return 0;
  const int rows = T;
  const Norm emb{we, inv_n, eps}, pre{wp, inv_n, eps};
#define OMNIA_EM(NT, N)                                                                            \
  do {                                                                                          \
    if (f32)                                                                                    \
      embed_kernel<float, NT, N><<<T, NT, 0, s>>>((float*)h, x, ids, (const float*)table, d,       \
                                               vocab, emb, pre, src, tok_slots);                \
    else                                                                                        \
      embed_kernel<bf16_t, NT, N><<<T, NT, 0, s>>>((bf16_t*)h, x, ids, (const bf16_t*)table, d,    \
                                                vocab, emb, pre, src, tok_slots);               \
  } while (0)
  OMNIA_NC(OMNIA_EM);
#undef OMNIA_EM
  return (int)hipGetLastError();
}

// ptype: storage of `m` -- 0 bf16, 1 fp32, 2 fp16 (slabs)
int omnia_rms_residual(void* h, int f32, float* x, const void* m, int ptype, int S,
                       int64_t row_stride, int64_t part_stride, int rows, int d,
                       const float* bias, const float* w_post, const float* w_pre, float inv_n, float eps,
                       hipStream_t s) {
  if (d % 4 || d < 4 || d > 16384 || S < 1 || row_stride % 4 || part_stride % 4 || !w_post)
    return -1;
  if (f32 && ptype != 1) return -2;
  if (rows == 0) return 0;
  const Norm post{w_post, inv_n, eps}, pre{w_pre, inv_n, eps};
#define OMNIA_RR(TT, PP, NT, N)                                                                 \
  residual_kernel<TT, PP, NT, N><<<rows, NT, 0, s>>>((TT*)h, x, (const PP*)m, S, row_stride,    \
                                                  part_stride, d, bias, post, pre)
#define OMNIA_RRN(NT, N)                                       \
  do {                                                      \
    if (f32) OMNIA_RR(float, float, NT, N);                     \
    else if (ptype == 0) OMNIA_RR(bf16_t, bf16_t, NT, N);       \
    else if (ptype == 1) OMNIA_RR(bf16_t, float, NT, N);        \
    else OMNIA_RR(bf16_t, _Float16, NT, N);                     \
  } while (0)
  OMNIA_NC(OMNIA_RRN);
#undef OMNIA_RRN
#undef OMNIA_RR
  return (int)hipGetLastError();
}

int omnia_softcap(void* z, int f32, int64_t n, float cap, hipStream_t s) {
  if (!(cap > 0.f)) return -1;
  if (n == 0) return 0;
  const int64_t want = (n / 4 + 255) / 256;
  const unsigned grid = (unsigned)(want < 1 ? 1 : want > 4096 ? 4096 : want);
  if (f32)
    softcap_kernel<float><<<grid, 256, 0, s>>>((float*)z, n, cap, 1.f / cap);
  else
    softcap_kernel<bf16_t><<<grid, 256, 0, s>>>((bf16_t*)z, n, cap, 1.f / cap);
  return (int)hipGetLastError();
}

}  // extern "C"
