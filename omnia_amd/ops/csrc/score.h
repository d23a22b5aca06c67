// What a query-key product becomes before the softmax: times scale, capped (cap tanh(s /
// cap)), then less a distance bias r1 ln(1 + r2 (i - j)) of its head.
#pragma once
#include "common.h"

namespace omnia {

struct Score {
  float scale;
  float cap;        // 0: none
  const float* r1;  // [H], or null: no bias
  const float* r2;

  __host__ bool ok() const { return cap >= 0.f && (r1 == nullptr) == (r2 == nullptr); }
  __host__ bool plain() const { return cap == 0.f && !r1; }

  // fp32 models
  __device__ __forceinline__ float operator()(float dot, int h, int distance) const {
    float s = dot * scale;
    if (cap > 0.f) s = cap * tanhf(s / cap);
    if (r1) s -= r1[h] * logf(1.f + r2[h] * (float)distance);
    return s;
  }
};

// bf16 kernels work in base 2: a score is log2(e) s.  With a cap,
// tanh(y) = 1 - 2 / (exp(2 y) + 1) on v_exp_f32 / v_rcp_f32.
struct Score2 {
  float mul;  // of the product: log2(e) scale, or with a cap 2 log2(e) scale / cap
  float cap;  // log2(e) cap, or 0
  const float* r1;
  const float* r2;

  __host__ explicit Score2(const Score& s) : r1(s.r1), r2(s.r2) {
    constexpr float log2e = 1.4426950408889634f;
    cap = log2e * s.cap;
    mul = s.cap > 0.f ? 2.f * log2e * s.scale / s.cap : log2e * s.scale;
  }
  // capped score of y = mul * product
  __device__ __forceinline__ float squash(float y) const {
    return __builtin_fmaf(-2.f * cap, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(y) + 1.f), cap);
  }
};

// log2(1 + r2 d) for an argument 1 + r2 d
__device__ __forceinline__ float log2_(float x) { return __builtin_amdgcn_logf(x); }

}  // namespace omnia
