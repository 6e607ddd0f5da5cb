// What the recurrent mixers' kernels share (ssm.hip, delta.hip): rows that a product left in the storage
// type, in float32 or as float32 partial sums; activations; the state of a short causal convolution.
#pragma once

#include "common.h"

namespace tk {

constexpr int kMaxTaps = 8;

// an input of [rows, ld] elements: T, or float32, or `parts` float32 partial sums `stride` elements apart
struct RowsIn {
  const void* p;
  int f32;
  int parts;
  long stride;
};

template <typename T>
__device__ __forceinline__ float load_in(const RowsIn& in, size_t idx) {
  if (!in.f32) return Elem<T>::load(reinterpret_cast<const T*>(in.p) + idx);
  const float* f = reinterpret_cast<const float*>(in.p) + idx;
  float s = f[0];
  int i = 1;
  for (; i + 3 < in.parts; i += 4) {      // four loads in flight; the sums in the order of the parts
    const float a = f[(size_t)i * in.stride], b = f[(size_t)(i + 1) * in.stride];
    const float c = f[(size_t)(i + 2) * in.stride], d = f[(size_t)(i + 3) * in.stride];
    s = (((s + a) + b) + c) + d;
  }
  for (; i < in.parts; ++i) s += f[(size_t)i * in.stride];
  return s;
}

__device__ __forceinline__ float sigmoid(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float silu(float x) { return x / (1.f + expf(-x)); }
// log(1 + e^x) = max(x, 0) + log1p(e), e = e^-|x|, with log1p(e) = log(u) e / (u - 1), u = 1 + e rounded (the rounding
// of u cancels in the quotient; the library's log1pf is several times the rest of a kernel that forms a decay
// per channel: 126 against 60 us for 2,048 tokens of 4,096 channels)
__device__ __forceinline__ float softplus(float x) {
  const float e = expf(-fabsf(x)), u = 1.f + e;
  return fmaxf(x, 0.f) + (u == 1.f ? e : __logf(u) * (e / (u - 1.f)));
}

// The state after a step: the last taps - 1 inputs of every request, from the step's rows or, where the
// step brought fewer, from the state before it.  A thread a (request, channel): it reads what it needs, then writes.
template <typename T>
__global__ __launch_bounds__(256) void conv_carry_kernel(
    RowsIn proj, long ld, int col0, float* __restrict__ state, const int* __restrict__ q_start,
    const int* __restrict__ state_slots, int C, int taps) {
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  const int req = blockIdx.y;
  if (c >= C) return;
  const int first = q_start[req], count = q_start[req + 1] - first;
  float* st = state + (size_t)state_slots[req] * (taps - 1) * C + c;
  float keep[kMaxTaps - 1];
#pragma unroll
  for (int j = 0; j < kMaxTaps - 1; ++j) {
    keep[j] = 0.f;
    if (j < taps - 1) {
      const int local = count - (taps - 1) + j;
      keep[j] = local >= 0 ? load_in<T>(proj, (size_t)(first + local) * ld + col0 + c) : st[(size_t)(taps - 1 + local) * C];
    }
  }
#pragma unroll
  for (int j = 0; j < kMaxTaps - 1; ++j)
    if (j < taps - 1) st[(size_t)j * C] = keep[j];
}

}  // namespace tk
