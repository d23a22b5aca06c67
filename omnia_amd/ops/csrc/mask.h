// Which keys a query at position p sees: its window [lo(p), p] and the sequence's kept
// first keys [0, kept).  Kernels walk the visible keys by an index that skips the gap.
#pragma once
#include "common.h"

namespace omnia {

struct Mask {
  int window;  // last `window` positions (0: the whole past)
  int keep;    // first positions every window also holds
  int chunk;   // > 0: the positions of p's own chunk, counted from position 0, instead

  __host__ bool ok() const { return window >= 0 && keep >= 0 && chunk >= 0; }
  // most keys a query sees of a context of n
  __host__ int most(int n) const {
    const int64_t m = chunk > 0 ? chunk : window > 0 ? (int64_t)window + keep : n;
    return m < n ? (int)m : n;
  }
  // first position of p's window (never decreases with p)
  __device__ __forceinline__ int lo(int p) const {
    if (chunk > 0) return p / chunk * chunk;
    return window > 0 ? max(0, p - window + 1) : 0;
  }
  // kept keys before a window that starts at lo
  __device__ __forceinline__ int kept(int lo) const { return chunk > 0 ? 0 : min(keep, lo); }
};

}  // namespace omnia
