// Linear attention with one constant decay a head, in chunks on the matrix cores (gfx950): the form of long portions.
//
//     S <- a S + k_t v_t^T,  o_t = S^T q_t,  q, k, v = silu(.) of the projection's columns [v | k | q | ...]
//
// A chunk of 64 tokens from position t0, with S its start state:
//     o_i = a^(i + 1) S^T q_i + sum_{j <= i} a^(i - j) (q_i . k_j) v_j,     S' = a^n S + sum_j a^(n - 1 - j) k_j v_j^T
// so a portion's chunks run side by side in three kernels: every chunk's own sum of k v^T (chunk_sums); per request the
// chunks in order, the start state of each, the request's new state (chunk_starts); every chunk's outputs
// (chunk_outputs).  Powers of a never exceed one.  All of it is float32: the products are the float32
// matrix instruction's (16 x 16 x 4), the operands are rounded nowhere behind the projection.
#include "common.h"
#include "short_conv.h"
#include "slots.h"

using namespace tk;

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int kChunk = 64;        // tokens of a chunk: four tiles of 16, one a wave
constexpr int kThreads = 256;
constexpr int kMaxDim = 128;

struct ChunkShape {
  int heads, dim, vdim;
  long ld;                        // columns of a projection row
  __host__ __device__ int dk() const { return (dim + 15) & ~15; }
  __host__ __device__ int dv() const { return (vdim + 15) & ~15; }
  __host__ __device__ int elems() const { return (vdim + 3) / 4 * dim * 4; }     // of a head's state: [column group][dim][4]
};

struct ChunkPlace {
  int first, count;               // the chunk's first token row, its tokens (0: there is no such chunk)
  size_t place;                   // its number among all chunks of the step, requests in order
};

__device__ __forceinline__ ChunkPlace chunk_place(const int* q_start, int max_chunks) {
  const int req = blockIdx.x / max_chunks, ci = blockIdx.x % max_chunks;
  const int first = q_start[req] + ci * kChunk, end = q_start[req + 1];
  int before = 0;
  for (int r = 0; r < req; ++r) before += (q_start[r + 1] - q_start[r] + kChunk - 1) / kChunk;
  return {first, max(0, min(kChunk, end - first)), (size_t)(before + ci)};
}

// silu of `width` columns from `col` on of the chunk's rows, times scale[row], into dst [64][pitch]; zeros elsewhere.
// WIDE: four neighbouring columns a piece (col, width and ld multiples of four).
template <typename T, bool WIDE, typename SCALE>
__device__ __forceinline__ void stage(float* dst, int pitch, const RowsIn& in, long ld, int col, int width, int padded,
                                      const ChunkPlace& c, SCALE scale) {
  const int quads = padded / 4;
  for (int e = threadIdx.x; e < kChunk * quads; e += kThreads) {
    const int t = e / quads, d = (e - t * quads) * 4;
    f32x4 v = {0.f, 0.f, 0.f, 0.f};
    if (t < c.count && d < width) {
      const size_t at = (size_t)(c.first + t) * ld + col + d;
      if (WIDE && !in.f32) {
        const uint2 u = *reinterpret_cast<const uint2*>(reinterpret_cast<const bf16_t*>(in.p) + at);
        v = f32x4{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
                  __uint_as_float(u.y & 0xffff0000u)};
      } else {
        v.x = load_in<T>(in, at);
        if (d + 1 < width) v.y = load_in<T>(in, at + 1);
        if (d + 2 < width) v.z = load_in<T>(in, at + 2);
        if (d + 3 < width) v.w = load_in<T>(in, at + 3);
      }
      const float s = scale(t);
      v = f32x4{silu(v.x) * s, silu(v.y) * s, silu(v.z) * s, silu(v.w) * s};
    }
    *reinterpret_cast<f32x4*>(dst + t * pitch + d) = v;
  }
}

// chunk_state[chunk][head] = sum_j a^(n - 1 - j) k_j v_j^T.  A block a (chunk, head); the tiles of 16 x 16 dealt to its waves.
template <typename T, bool WIDE>
__global__ __launch_bounds__(kThreads) void chunk_sums_kernel(RowsIn in, const float* __restrict__ decay,
                                                              const int* __restrict__ q_start, float* __restrict__ chunk_state,
                                                              ChunkShape sh, int max_chunks) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const ChunkPlace c = chunk_place(q_start, max_chunks);
  if (c.count == 0) return;       // (the whole block, before any barrier)
  const int head = blockIdx.y, dk = sh.dk(), dv = sh.dv(), kp = dk + 4, vp = dv + 4;
  float* kk = lds;
  float* vv = kk + kChunk * kp;
  float* pw = vv + kChunk * vp;
  const float a = decay[head];
  if (threadIdx.x < kChunk) pw[threadIdx.x] = powf(a, (float)threadIdx.x);
  __syncthreads();
  stage<T, WIDE>(kk, kp, in, sh.ld, sh.heads * sh.vdim + head * sh.dim, sh.dim, dk, c, [&](int t) { return pw[c.count - 1 - t]; });
  stage<T, WIDE>(vv, vp, in, sh.ld, head * sh.vdim, sh.vdim, dv, c, [](int) { return 1.f; });
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, col = lane & 15, quad = lane >> 4;
  const int tiles = (dk / 16) * (dv / 16), steps = (c.count + 3) / 4;
  float* out = chunk_state + (c.place * sh.heads + head) * (size_t)sh.elems();
  for (int tile = wave; tile < tiles; tile += kThreads / 64) {
    const int d0 = tile / (dv / 16) * 16, v0 = tile % (dv / 16) * 16;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int s = 0; s < steps; ++s)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kk[(s * 4 + quad) * kp + d0 + col], vv[(s * 4 + quad) * vp + v0 + col], acc, 0, 0, 0);
    const int v = v0 + col;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = d0 + quad * 4 + r;
      if (d < sh.dim && v < (sh.vdim + 3) / 4 * 4) out[((size_t)(v >> 2) * sh.dim + d) * 4 + (v & 3)] = acc[r];   // (columns behind vdim: zeros)
    }
  }
}

// Per (request, head), a thread an element of the state: chunk_state holds every chunk's own sum on entry and its start
// state on return; the request's state moves to the end of the step's tokens.
__global__ __launch_bounds__(256) void chunk_starts_kernel(float* __restrict__ state, const float* __restrict__ decay,
                                                           const int* __restrict__ q_start, const int* __restrict__ state_slots,
                                                           float* __restrict__ chunk_state, int heads, int elems) {
  const int req = blockIdx.x, head = blockIdx.y;
  const int tokens = q_start[req + 1] - q_start[req], count = (tokens + kChunk - 1) / kChunk;
  int before = 0;
  for (int r = 0; r < req; ++r) before += (q_start[r + 1] - q_start[r] + kChunk - 1) / kChunk;
  const float a = decay[head], whole = powf(a, (float)kChunk), last = powf(a, (float)(tokens - (count - 1) * kChunk));
  const int e = blockIdx.z * blockDim.x + threadIdx.x;
  if (e >= elems) return;
  float* S = state + ((size_t)state_slots[req] * heads + head) * elems + e;
  float* cs = chunk_state + ((size_t)before * heads + head) * elems + e;
  const size_t stride = (size_t)heads * elems;
  float s = *S;
  for (int c0 = 0; c0 < count; c0 += 8) {       // eight chunks' sums in flight
    float own[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) own[u] = c0 + u < count ? cs[(c0 + u) * stride] : 0.f;
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      if (c0 + u < count) {
        cs[(c0 + u) * stride] = s;
        s = fmaf(c0 + u == count - 1 ? last : whole, s, own[u]);
      }
    }
  }
  *S = s;
}

// The outputs of a chunk.  A block a (chunk, head), wave w the tokens 16 w .. + 16.
template <typename T, bool WIDE>
__global__ __launch_bounds__(kThreads) void chunk_outputs_kernel(RowsIn in, const float* __restrict__ decay,
                                                                 const int* __restrict__ q_start,
                                                                 const float* __restrict__ chunk_state, float* __restrict__ y,
                                                                 ChunkShape sh, int max_chunks) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const ChunkPlace c = chunk_place(q_start, max_chunks);
  if (c.count == 0) return;       // (the whole block, before any barrier)
  constexpr int PP = kChunk + 4;
  const int head = blockIdx.y, dk = sh.dk(), dv = sh.dv(), kp = dk + 4, vp = dv + 4;
  float* qq = lds;
  float* kk = qq + kChunk * kp;   // the keys, then the weighted scores [64][PP]
  float* vv = kk + kChunk * max(kp, PP);
  float* pw = vv + kChunk * vp;
  const float a = decay[head];
  if (threadIdx.x <= kChunk) pw[threadIdx.x] = powf(a, (float)threadIdx.x);
  const int kcol = sh.heads * sh.vdim + head * sh.dim;
  const auto one = [](int) { return 1.f; };
  stage<T, WIDE>(qq, kp, in, sh.ld, kcol + sh.heads * sh.dim, sh.dim, dk, c, one);
  stage<T, WIDE>(kk, kp, in, sh.ld, kcol, sh.dim, dk, c, one);
  stage<T, WIDE>(vv, vp, in, sh.ld, head * sh.vdim, sh.vdim, dv, c, one);
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, col = lane & 15, quad = lane >> 4;
  const bool works = wave * 16 < c.count;
  const float* q_row = qq + (wave * 16 + col) * kp + quad;
  f32x4 score[kChunk / 16];
#pragma unroll
  for (int jt = 0; jt < kChunk / 16; ++jt) {
    score[jt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (works && jt <= wave) {
      const float* k_row = kk + (jt * 16 + col) * kp + quad;
#pragma unroll 4
      for (int d = 0; d < dk; d += 4) score[jt] = __builtin_amdgcn_mfma_f32_16x16x4f32(q_row[d], k_row[d], score[jt], 0, 0, 0);
    }
  }
  __syncthreads();                // (every wave has read its keys: their place takes the scores)
#pragma unroll
  for (int jt = 0; jt < kChunk / 16; ++jt) {
    if (works && jt <= wave) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = wave * 16 + quad * 4 + r, j = jt * 16 + col;
        kk[i * PP + j] = j <= i ? score[jt][r] * pw[i - j] : 0.f;
      }
    }
  }
  wave_lds_sync();                // (a wave reads back its own rows only)
  if (!works) return;
  const float* p_row = kk + (wave * 16 + col) * PP + quad;
  const float* S = chunk_state + (c.place * sh.heads + head) * (size_t)sh.elems();
  const int groups = (sh.vdim + 3) / 4;
  for (int v0 = 0; v0 < dv; v0 += 16) {
    const int v = v0 + col;
    const float* s_col = S + ((size_t)min(v >> 2, groups - 1) * sh.dim) * 4 + (v & 3);    // (columns behind the last group are not stored)
    f32x4 far = {0.f, 0.f, 0.f, 0.f}, near = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int d = 0; d < dk; d += 4) {
      const float b = d + quad < sh.dim ? s_col[(d + quad) * 4] : 0.f;
      far = __builtin_amdgcn_mfma_f32_16x16x4f32(q_row[d], b, far, 0, 0, 0);
    }
#pragma unroll 4
    for (int j = 0; j < (wave + 1) * 16; j += 4)
      near = __builtin_amdgcn_mfma_f32_16x16x4f32(p_row[j], vv[(j + quad) * vp + v], near, 0, 0, 0);
    if (v < sh.vdim) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = wave * 16 + quad * 4 + r;
        if (i < c.count) y[(size_t)(c.first + i) * sh.heads * sh.vdim + (size_t)head * sh.vdim + v] = fmaf(pw[i + 1], far[r], near[r]);
      }
    }
  }
}

template <typename T, bool WIDE>
int launch(RowsIn in, const float* decay, float* state, const int* q_start, const int* slots, float* y, int R, ChunkShape sh,
           int max_chunks, float* chunk_state, hipStream_t stream) {
  const int kp = sh.dk() + 4, vp = sh.dv() + 4;
  const size_t sums_lds = ((size_t)kChunk * (kp + vp) + kChunk) * 4;
  const size_t out_lds = ((size_t)kChunk * (kp + max(kp, kChunk + 4) + vp) + kChunk + 1) * 4;
  static bool raised = false;
  if (!raised) {
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(&chunk_sums_kernel<T, WIDE>), hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024) != hipSuccess ||
        hipFuncSetAttribute(reinterpret_cast<const void*>(&chunk_outputs_kernel<T, WIDE>), hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024) != hipSuccess)
      return -1;
    raised = true;
  }
  const dim3 grid(R * max_chunks, sh.heads);
  chunk_sums_kernel<T, WIDE><<<grid, kThreads, sums_lds, stream>>>(in, decay, q_start, chunk_state, sh, max_chunks);
  chunk_starts_kernel<<<dim3(R, sh.heads, (sh.elems() + 255) / 256), 256, 0, stream>>>(state, decay, q_start, slots, chunk_state,
                                                                                       sh.heads, sh.elems());
  chunk_outputs_kernel<T, WIDE><<<grid, kThreads, out_lds, stream>>>(in, decay, q_start, chunk_state, y, sh, max_chunks);
  return launch_status();
}

}  // namespace

// proj, decay, state and y as in tk_fixed_decay_scan (ssm.hip), dim and vdim up to 128; max_chunks: the most chunks of 64
// tokens a request of the step has; chunk_state float32 [chunks of the step, heads, ceil(vdim / 4), dim, 4] is scratch.
TK_API int tk_fixed_decay_chunks(int dtype, const void* proj, int in_f32, int parts, long part_stride, long ld,
                                 const float* decay, float* state, const int* q_start, const int* state_slots, float* y,
                                 int R, int heads, int dim, int vdim, int max_chunks, float* chunk_state, hipStream_t stream) {
  if (R <= 0) return 0;
  if (heads < 1 || heads > 65535 || dim < 1 || dim > kMaxDim || vdim < 1 || vdim > kMaxDim || max_chunks < 1 ||
      (long)R * max_chunks > 0x7fffffffL || parts < 1 || (parts > 1 && !in_f32) || ld < (long)heads * (vdim + 2 * dim) ||
      chunk_state == nullptr)
    return -1;
  const RowsIn in{proj, in_f32 || dtype == 0, parts, part_stride};
  const ChunkShape sh{heads, dim, vdim, ld};
  const bool wide = dim % 4 == 0 && vdim % 4 == 0 && ld % 4 == 0 && (uintptr_t)proj % 16 == 0;
  if (dtype == 0) return launch<float, false>(in, decay, state, q_start, state_slots, y, R, sh, max_chunks, chunk_state, stream);
  if (wide) return launch<bf16_t, true>(in, decay, state, q_start, state_slots, y, R, sh, max_chunks, chunk_state, stream);
  return launch<bf16_t, false>(in, decay, state, q_start, state_slots, y, R, sh, max_chunks, chunk_state, stream);
}

TK_SLOTS(tk_fixed_decay_chunks)
