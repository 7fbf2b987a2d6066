// window_common.h -- which keys a query sees: a window and kept first tokens.
#pragma once
#include "latent/latent_common.h"
#include "slm_mixers.h"

namespace slm {

// The visible positions of a query at p as one index range [0, count): kept first tokens, then the window.
struct VisibleKeys {
  int kept, lo, count;
  __device__ __forceinline__ VisibleKeys(int p, int window, int keep_first) {
    lo = window > 0 ? max(0, p - window + 1) : 0;
    kept = min(max(keep_first, 0), lo);
    count = kept + p - lo + 1;
  }
  __device__ __forceinline__ int position(int i) const { return i < kept ? i : lo + i - kept; }
};

__device__ __forceinline__ bool key_visible(int q, int k, int window, int keep_first) {
  return k <= q && (window <= 0 || q - k < window || k < keep_first);
}

}  // namespace slm
