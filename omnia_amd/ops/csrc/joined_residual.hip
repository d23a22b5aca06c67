// Residual step of a layer whose sublayers read the same residual (bf16 or fp32 models, fp32
// residual), in one pass:
//
//     x += sum of the sublayers' parts [ + scale * embedding + step ]
//     h1 = rms(x) * g1 * w1 ,  h2 = rms(x) * g2 * w2      (one mean, one or two norms)
//
// Up to three parts: a projection or its split-K slabs (the mixer's output, a dense or shared
// feed-forward), and the slots of a token's experts.  The bracket is what a pass of a looped
// stretch enters with: the embedding row of the row's token, gathered again, and a vector.
// With x starting from zero and no parts, that is the embedding step of the model.
//
// One workgroup per row; a thread keeps its columns in registers.  First loads of all
// operands are issued raw before any is converted, so that they are in flight together.
#include "common.h"

using namespace omnia;

namespace {

typedef _Float16 half4v __attribute__((ext_vector_type(4)));

// storage 0 bf16, 1 fp32, 2 fp16
template <int P>
struct Raw4;
template <>
struct Raw4<0> {
  typedef short4v t;
  typedef bf16_t e;
};
template <>
struct Raw4<1> {
  typedef float4v t;
  typedef float e;
};
template <>
struct Raw4<2> {
  typedef half4v t;
  typedef _Float16 e;
};
__device__ __forceinline__ float4v wide(short4v h) {
  return float4v{bf2f((uint16_t)h[0]), bf2f((uint16_t)h[1]), bf2f((uint16_t)h[2]),
                 bf2f((uint16_t)h[3])};
}
__device__ __forceinline__ float4v wide(float4v v) { return v; }
__device__ __forceinline__ float4v wide(half4v h) {
  return float4v{(float)h[0], (float)h[1], (float)h[2], (float)h[3]};
}
template <int P>
__device__ __forceinline__ typename Raw4<P>::t raw4(const void* base, int64_t at) {
  return *reinterpret_cast<const typename Raw4<P>::t*>((const typename Raw4<P>::e*)base + at);
}
__device__ __forceinline__ void store4(float* p, float4v v) { *reinterpret_cast<float4v*>(p) = v; }
__device__ __forceinline__ void store4(bf16_t* p, float4v v) {
  uint2v k;
  k[0] = pack_bf2(v[0], v[1]);
  k[1] = pack_bf2(v[2], v[3]);
  *reinterpret_cast<uint2v*>(p) = k;
}

struct Part {  // S 0: absent
  const void* m;
  int type, S;
  int64_t row, part;
};
struct Enter {
  const int* ids;
  const void* table;  // null: no embedding; rows of the model's type
  int vocab;
  float scale;
  const float* step;  // or null
  const int64_t* src;
  const int* tok_slots;
};
struct Norm {
  const float* w;  // or null
  float gain;
};

// the parts past the first U (already added), four in flight
template <int P, int U, int NT, int NC>
__device__ __forceinline__ void rest(float4v (&v)[NC], const Part& p, int64_t t, int d) {
  const float4v zero = {0.f, 0.f, 0.f, 0.f};
  for (int s = U; s < p.S; s += 4) {
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int c = (threadIdx.x + i * NT) * 4;
      if (c < d) {
        float4v q[4];
#pragma unroll
        for (int j = 0; j < 4; ++j)
          q[j] = s + j < p.S ? wide(raw4<P>(p.m, t * p.row + (s + j) * p.part + c)) : zero;
        v[i] += (q[0] + q[1]) + (q[2] + q[3]);
      }
    }
  }
}

// T, PT: the model's type and its storage number; part b is stored in it
template <typename T, int PT, int PA, int PC, int NT, int NC>
__global__ __launch_bounds__(NT) void joined_kernel(T* __restrict__ h1, T* __restrict__ h2,
                                                    float* __restrict__ x, int fresh, int d,
                                                    Part a, Part b, Part c, Enter en, Norm n1,
                                                    Norm n2, float inv_n, float eps) {
  __shared__ float scratch[NT / 64];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x;
  int64_t erow = -1;
  if (en.table) {
    const int64_t sl = en.src ? en.src[t] : -1;
    const int id = sl >= 0 ? en.tok_slots[sl] : en.ids[t];
    if (id >= 0 && id < en.vocab) erow = id;
  }
  float4v old[NC];
  typename Raw4<PA>::t ra[NC];
  typename Raw4<PT>::t rb[2][NC], re[NC];
  typename Raw4<PC>::t rc[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int col = (tid + i * NT) * 4;
    const bool in = col < d;
    old[i] = float4v{0.f, 0.f, 0.f, 0.f};
    ra[i] = typename Raw4<PA>::t{0, 0, 0, 0};
    rc[i] = typename Raw4<PC>::t{0, 0, 0, 0};
    rb[0][i] = rb[1][i] = re[i] = typename Raw4<PT>::t{0, 0, 0, 0};
    if (in && !fresh) old[i] = *reinterpret_cast<const float4v*>(x + t * d + col);
    if (in && a.S > 0) ra[i] = raw4<PA>(a.m, t * a.row + col);
    if (in && b.S > 0) rb[0][i] = raw4<PT>(b.m, t * b.row + col);
    if (in && b.S > 1) rb[1][i] = raw4<PT>(b.m, t * b.row + b.part + col);
    if (in && c.S > 0) rc[i] = raw4<PC>(c.m, t * c.row + col);
    if (in && erow >= 0) re[i] = raw4<PT>(en.table, erow * d + col);
  }
  float4v v[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i)
    v[i] = (wide(ra[i]) + wide(rc[i])) + (wide(rb[0][i]) + wide(rb[1][i]));
  rest<PA, 1, NT, NC>(v, a, t, d);
  rest<PT, 2, NT, NC>(v, b, t, d);
  rest<PC, 1, NT, NC>(v, c, t, d);
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int col = (tid + i * NT) * 4;
    v[i] += old[i] + en.scale * wide(re[i]);
    if (col < d) {
      if (en.step) v[i] += *reinterpret_cast<const float4v*>(en.step + col);
      store4(x + t * d + col, v[i]);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) ss += v[i][j] * v[i][j];
  }
  ss = block_sum(ss, scratch);
  const float r = 1.f / sqrtf(ss * inv_n + eps);
  auto put = [&](T* h, const Norm& n) {
#pragma unroll
    for (int i = 0; i < NC; ++i) {
      const int col = (tid + i * NT) * 4;
      if (col < d) {
        float4v y = v[i] * (r * n.gain);
        if (n.w) y *= *reinterpret_cast<const float4v*>(n.w + col);
        store4(h + t * d + col, y);
      }
    }
  };
  put(h1, n1);
  if (h2) put(h2, n2);
}

}  // namespace

// parts a and c: any storage; part b: the model's.  S 0: absent
extern "C" int omnia_joined_residual(void* h1, void* h2, int f32, float* x, int fresh, int rows,
                                     int d, const void* am, int at, int aS, int64_t arow,
                                     int64_t apart, const void* bm, int bS, int64_t brow,
                                     int64_t bpart, const void* cm, int ct, int cS, int64_t crow,
                                     int64_t cpart, const int* ids, const void* table, int vocab,
                                     float scale, const float* step, const int64_t* src,
                                     const int* tok_slots, const float* w1, float g1,
                                     const float* w2, float g2, float inv_n, float eps,
                                     hipStream_t s) {
  if (d % 4 || d < 4 || d > 16384 || aS < 0 || bS < 0 || cS < 0 || arow % 4 || apart % 4 ||
      brow % 4 || bpart % 4 || crow % 4 || cpart % 4)
    return -1;
  if (at < 0 || at > 2 || ct < 0 || ct > 2 || (f32 && (at != 1 || ct != 1))) return -2;
  if (table && !ids) return -3;
  if (src && !tok_slots) return -4;
  if (rows == 0) return 0;
  const Part a{am, at, aS, arow, apart}, b{bm, f32, bS, brow, bpart}, c{cm, ct, cS, crow, cpart};
  const Enter en{ids, table, vocab, table ? scale : 0.f, step, src, tok_slots};
  const Norm n1{w1, g1}, n2{w2, g2};
#define OMNIA_JR(TT, PT, PA, PC, NT, NC)                                                      \
  joined_kernel<TT, PT, PA, PC, NT, NC><<<rows, NT, 0, s>>>((TT*)h1, (TT*)h2, x, fresh, d, a, \
                                                            b, c, en, n1, n2, inv_n, eps)
#define OMNIA_JRC(PA, NT, NC)                              \
  do {                                                     \
    if (ct == 0) OMNIA_JR(bf16_t, 0, PA, 0, NT, NC);       \
    else if (ct == 1) OMNIA_JR(bf16_t, 0, PA, 1, NT, NC);  \
    else OMNIA_JR(bf16_t, 0, PA, 2, NT, NC);               \
  } while (0)
#define OMNIA_JRN(NT, NC)                                  \
  do {                                                     \
    if (f32) OMNIA_JR(float, 1, 1, 1, NT, NC);             \
    else if (at == 0) OMNIA_JRC(0, NT, NC);                \
    else if (at == 1) OMNIA_JRC(1, NT, NC);                \
    else OMNIA_JRC(2, NT, NC);                             \
  } while (0)
  if (d <= 1024) OMNIA_JRN(256, 1);
  else if (rows <= 512 && d <= 4096) OMNIA_JRN(1024, 1);
  else if (d <= 2048) OMNIA_JRN(256, 2);
  else if (d <= 4096) OMNIA_JRN(512, 2);
  else if (d <= 8192) OMNIA_JRN(1024, 2);
  else OMNIA_JRN(1024, 4);
#undef OMNIA_JRN
#undef OMNIA_JRC
#undef OMNIA_JR
  return (int)hipGetLastError();
}
