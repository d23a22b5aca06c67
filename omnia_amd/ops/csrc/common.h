// Shared device helpers for the omnia_amd CDNA4 (gfx950) kernels.
//
// Everything here is written for 64-lane wavefronts and the gfx950 MFMA /
// LDS model (see docs/KERNELS.md).  No CUDA spellings, no dual paths.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace omnia {

using bf16_t = uint16_t;  // raw bf16 storage
typedef short short8 __attribute__((ext_vector_type(8)));
typedef short short4v __attribute__((ext_vector_type(4)));
typedef float float4v __attribute__((ext_vector_type(4)));
typedef float float16v __attribute__((ext_vector_type(16)));
typedef unsigned int uint4v __attribute__((ext_vector_type(4)));
typedef unsigned int uint2v __attribute__((ext_vector_type(2)));

constexpr int kWave = 64;

__device__ __forceinline__ float bf2f(uint16_t x) {
  return __uint_as_float(((uint32_t)x) << 16);
}

// round-to-nearest-even f32 -> bf16 (inputs are finite on every hot path)
__device__ __forceinline__ uint16_t f2bf(float f) {
  uint32_t u = __float_as_uint(f);
  u += 0x7fffu + ((u >> 16) & 1u);
  return (uint16_t)(u >> 16);
}

// two f32 -> packed bf16x2 (low = a)
__device__ __forceinline__ uint32_t pack_bf2(float a, float b) {
  return (uint32_t)f2bf(a) | ((uint32_t)f2bf(b) << 16);
}

// element access of kernels instantiated for bf16 (serving) and fp32 storage
__device__ __forceinline__ float ldf(const bf16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ldf(const float* p) { return *p; }
__device__ __forceinline__ float ldf(const _Float16* p) { return (float)*p; }
__device__ __forceinline__ void stf(bf16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void stf(float* p, float v) { *p = v; }

// fp32 to a few ulp (v_exp_f32 / v_rcp_f32)
__device__ __forceinline__ float sigmoidf_(float x) {
  return __builtin_amdgcn_rcpf(1.f + __expf(-x));
}
__device__ __forceinline__ float siluf_(float x) { return x * sigmoidf_(x); }
// gelu, tanh form: 0.5 x (1 + tanh(y)) = x sigmoid(2 y)
__device__ __forceinline__ float gelu_tanh_(float x) {
  return x * sigmoidf_(1.5957691216057308f * (x + 0.044715f * x * x * x));
}
// gelu, erf form, for 16-bit results: max(x, 0) - |x| e, e = 0.5 erfc(|x| / sqrt(2)) by
// Abramowitz and Stegun 7.1.26 (|error| of erf < 1.5e-7), its constants scaled to |x|
__device__ __forceinline__ float gelu_erf16_(float x) {
  const float a = fabsf(x), t = __builtin_amdgcn_rcpf(1.f + 0.23164189f * a);
  const float p = ((((0.5307027145f * t - 0.7265760135f) * t + 0.7107068705f) * t -
                    0.142248368f) * t + 0.127414796f) * t;
  return fmaxf(x, 0.f) - a * p * __builtin_amdgcn_exp2f(-0.7213475204f * x * x);
}
// gelu, erf form
__device__ __forceinline__ float gelu_erf_(float x) {
  return 0.5f * x * (1.f + erff(x * 0.7071067811865476f));
}

// sum over the 16 lanes of a DPP row, result in every lane of the row
template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
  return v + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float row_sum16(float v) {
  v = dpp_add<0xB1>(v);      // quad_perm: xor 1
  v = dpp_add<0x4E>(v);      // quad_perm: xor 2
  v = dpp_add<0x141>(v);     // row_half_mirror
  return dpp_add<0x140>(v);  // row_mirror
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
  return v;
}

// block-wide sum; `scratch` holds >= blockDim/64 floats
__device__ __forceinline__ float block_sum(float v, float* scratch) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int nw = (blockDim.x + 63) >> 6;
  v = wave_sum(v);
  __syncthreads();
  if (lane == 0) scratch[wid] = v;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < nw; ++i) t += scratch[i];
  return t;
}

__device__ __forceinline__ float block_max(float v, float* scratch) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int nw = (blockDim.x + 63) >> 6;
  v = wave_max(v);
  __syncthreads();
  if (lane == 0) scratch[wid] = v;
  __syncthreads();
  float t = -INFINITY;
  for (int i = 0; i < nw; ++i) t = fmaxf(t, scratch[i]);
  return t;
}

// 64-bit mix (splitmix64 finaliser) -> counter-based RNG for the sampler
__device__ __forceinline__ uint64_t mix64(uint64_t z) {
  z += 0x9e3779b97f4a7c15ull;
  z = (z ^ (z >> 30)) * 0xbf58476d1ce4e5b9ull;
  z = (z ^ (z >> 27)) * 0x94d049bb133111ebull;
  return z ^ (z >> 31);
}

__device__ __forceinline__ float uniform01(uint64_t seed, uint64_t ctr) {
  uint64_t r = mix64(seed ^ mix64(ctr));
  // 24 random mantissa bits, strictly inside (0,1)
  return ((float)(r >> 40) + 0.5f) * (1.0f / 16777216.0f);
}

// XCD-aware bijective remap of a 1-D block id: blocks b and b+8 share an XCD
// under round-robin dispatch; give each XCD a contiguous chunk of the logical
// grid so neighbouring tiles share its L2 (guide T1, bijective form).
__device__ __forceinline__ int xcd_remap(int orig, int nwg) {
  const int q = nwg >> 3, r = nwg & 7, xcd = orig & 7;
  return (xcd < r ? xcd * (q + 1) : r * (q + 1) + (xcd - r) * q) + (orig >> 3);
}

}  // namespace omnia
