#pragma once

#include <hip/hip_runtime.h>

namespace tk {

// Attention scores bounded softly: s <- cap tanh(s / cap), formed in units of log2 as the softmax kernels keep
// them.  With x the raw product q . k, tanh(z) = 1 - 2 / (exp(2 z) + 1) gives
// log2(e) cap tanh(scale x / cap) = post - 2 post / (exp2(pre x) + 1).
struct SoftCap {
  float pre, post;      // 2 log2(e) scale / cap, log2(e) cap
  __device__ __forceinline__ float log2_score(float x) const {
    return fmaf(-2.f * post, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(x * pre) + 1.f), post);
  }
};
inline SoftCap soft_cap(float scale, float cap) {
  return cap > 0.f ? SoftCap{2.f * 1.4426950408889634f * scale / cap, 1.4426950408889634f * cap} : SoftCap{0.f, 0.f};
}

}  // namespace tk
