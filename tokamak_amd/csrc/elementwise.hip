// Memory-bound kernels of one step: embedding gather, residual add + RMSNorm,
// rotary tables, per-head q/k norm + rotation + cache write, SiLU-gate product.
// The residual stream is float32 in both dtypes; norm statistics, rotation
// angles and the residual sum are float32.
#include "common.h"
#include "slots.h"

using namespace tk;

// four neighbouring elements as floats, one access
template <typename TD> struct Load4;
template <> struct Load4<float> {
  static __device__ __forceinline__ float4 at(const float* p) { return *reinterpret_cast<const float4*>(p); }
};
template <> struct Load4<bf16_t> {
  static __device__ __forceinline__ float4 at(const bf16_t* p) {
    const uint2 u = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u),
                       __uint_as_float(u.y << 16), __uint_as_float(u.y & 0xffff0000u));
  }
};
template <typename T> struct Store4;
template <> struct Store4<float> {
  static __device__ __forceinline__ void at(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
};
template <> struct Store4<bf16_t> {
  static __device__ __forceinline__ void at(bf16_t* p, float4 v) {
    uint2 u;
    u.x = pack_bf16x2(v.x, v.y);
    u.y = pack_bf16x2(v.z, v.w);
    *reinterpret_cast<uint2*>(p) = u;
  }
};

// ---------------------------------------------------------------------------
// embedding: resid[n, :] = float(table[ids[n], :]) * scale, or with `accumulate`
// resid[n, :] += float(table[ids[n], :]) * scale (the same rows added to the stream once
// more, for a model that feeds its input in again); an id outside [0, V) gives NaN
// ---------------------------------------------------------------------------
template <typename T>
__global__ void embed_gather_kernel(const T* __restrict__ table, const int* __restrict__ ids,
                                    float* __restrict__ resid, int H, int V, float scale, int accumulate) {
  const int n = blockIdx.x;
  const int id = ids[n];
  float* out = resid + (size_t)n * H;
  if (id < 0 || id >= V) {
    for (int d = threadIdx.x; d < H; d += blockDim.x) out[d] = __uint_as_float(0x7fc00000u);
    return;
  }
  const T* row = table + (size_t)id * H;
  if (accumulate) {
    for (int d = threadIdx.x; d < H; d += blockDim.x) out[d] += Elem<T>::load(row + d) * scale;
  } else {
    for (int d = threadIdx.x; d < H; d += blockDim.x) out[d] = Elem<T>::load(row + d) * scale;
  }
}

TK_API int tk_embed_gather(int dtype, const void* table, const int* ids, float* resid, int N, int H,
                           int V, float scale, int accumulate, hipStream_t stream) {
  if (N <= 0) return 0;
  if (dtype == 0)
    embed_gather_kernel<float><<<N, 256, 0, stream>>>((const float*)table, ids, resid, H, V, scale, accumulate);
  else
    embed_gather_kernel<bf16_t><<<N, 256, 0, stream>>>((const bf16_t*)table, ids, resid, H, V, scale, accumulate);
  return launch_status();
}

// resid[n, :] (+)= r / sqrt(mean(r^2) + eps) * weight with r = float(table[ids[n], :]) * scale: an embedding with a
// norm of its own.  A block a token; the row is read twice (the second time from the cache).
template <typename T>
__global__ __launch_bounds__(256) void embed_norm_kernel(const T* __restrict__ table, const int* __restrict__ ids,
                                                         const float* __restrict__ weight, float* __restrict__ resid,
                                                         int H, int V, float scale, float eps, int accumulate) {
  __shared__ float scratch[16];
  const int n = blockIdx.x;
  const int id = ids[n];
  float* out = resid + (size_t)n * H;
  if (id < 0 || id >= V) {      // (the whole block, before any barrier)
    for (int d = threadIdx.x; d < H; d += blockDim.x) out[d] = __uint_as_float(0x7fc00000u);
    return;
  }
  const T* row = table + (size_t)id * H;
  float ss = 0.f;
  for (int d = threadIdx.x; d < H; d += blockDim.x) {
    const float v = Elem<T>::load(row + d) * scale;
    ss = fmaf(v, v, ss);
  }
  ss = block_sum(ss, scratch);
  const float rstd = 1.f / sqrtf(ss / (float)H + eps);
  for (int d = threadIdx.x; d < H; d += blockDim.x) {
    const float v = Elem<T>::load(row + d) * scale * rstd * weight[d];
    out[d] = accumulate ? out[d] + v : v;
  }
}

// The same, the row in registers: H a multiple of 4 and at most 16 * blockDim.
template <typename T>
__global__ __launch_bounds__(1024) void embed_norm_vec_kernel(const T* __restrict__ table, const int* __restrict__ ids,
                                                              const float* __restrict__ weight, float* __restrict__ resid,
                                                              int H, int V, float scale, float eps, int accumulate) {
  constexpr int GROUPS = 4;
  __shared__ float scratch[16];
  const int n = blockIdx.x;
  const int id = ids[n];
  float* out = resid + (size_t)n * H;
  if (id < 0 || id >= V) {      // (the whole block, before any barrier)
    for (int d = threadIdx.x; d < H; d += blockDim.x) out[d] = __uint_as_float(0x7fc00000u);
    return;
  }
  const T* row = table + (size_t)id * H;
  float4 v[GROUPS], w[GROUPS];
  float ss = 0.f;
#pragma unroll
  for (int g = 0; g < GROUPS; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    v[g] = w[g] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (d < H) {
      v[g] = Load4<T>::at(row + d);
      w[g] = *reinterpret_cast<const float4*>(weight + d);
    }
  }
#pragma unroll
  for (int g = 0; g < GROUPS; ++g) {
    v[g].x *= scale; v[g].y *= scale; v[g].z *= scale; v[g].w *= scale;
    ss += v[g].x * v[g].x + v[g].y * v[g].y + v[g].z * v[g].z + v[g].w * v[g].w;
  }
  ss = block_sum(ss, scratch);
  const float rstd = 1.f / sqrtf(ss / (float)H + eps);
#pragma unroll
  for (int g = 0; g < GROUPS; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    if (d < H) {
      float4 o = make_float4(v[g].x * rstd * w[g].x, v[g].y * rstd * w[g].y, v[g].z * rstd * w[g].z, v[g].w * rstd * w[g].w);
      if (accumulate) {
        const float4 x = *reinterpret_cast<const float4*>(out + d);
        o.x += x.x; o.y += x.y; o.z += x.z; o.w += x.w;
      }
      *reinterpret_cast<float4*>(out + d) = o;
    }
  }
}

TK_API int tk_embed_norm(int dtype, const void* table, const int* ids, const float* weight, float* resid, int N, int H,
                         int V, float scale, float eps, int accumulate, hipStream_t stream) {
  if (N <= 0) return 0;
  int threads = 64;
  while (threads < 1024 && threads * 4 < H) threads *= 2;
  if (H % 4 == 0 && H <= threads * 16 && (uintptr_t)table % 16 == 0 && (uintptr_t)weight % 16 == 0 && (uintptr_t)resid % 16 == 0) {
    if (dtype == 0)
      embed_norm_vec_kernel<float><<<N, threads, 0, stream>>>((const float*)table, ids, weight, resid, H, V, scale, eps, accumulate);
    else
      embed_norm_vec_kernel<bf16_t><<<N, threads, 0, stream>>>((const bf16_t*)table, ids, weight, resid, H, V, scale, eps, accumulate);
    return launch_status();
  }
  if (dtype == 0)
    embed_norm_kernel<float><<<N, 256, 0, stream>>>((const float*)table, ids, weight, resid, H, V, scale, eps, accumulate);
  else
    embed_norm_kernel<bf16_t><<<N, 256, 0, stream>>>((const bf16_t*)table, ids, weight, resid, H, V, scale, eps, accumulate);
  return launch_status();
}

// ---------------------------------------------------------------------------
// Token ids that are still on the GPU: ids[slots[i]] = sampled[rows[i]].  A step may be
// launched before the host has read the tokens that the step before it sampled; its
// descriptor then names, for such a token, the row of the sampler's output to take it from.
// ---------------------------------------------------------------------------
__global__ void feed_tokens_kernel(int* __restrict__ ids, const int* __restrict__ sampled,
                                   const int* __restrict__ slots, const int* __restrict__ rows, int count) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i < count) ids[slots[i]] = sampled[rows[i]];
}

TK_API int tk_feed_tokens(int* ids, const int* sampled, const int* slots, const int* rows, int count,
                          hipStream_t stream) {
  if (count <= 0) return 0;
  feed_tokens_kernel<<<(count + 255) / 256, 256, 0, stream>>>(ids, sampled, slots, rows, count);
  return launch_status();
}

// ---------------------------------------------------------------------------
// residual add + RMSNorm over rows of width H.
//   x = resid[row] (+ delta[row]);  if write_resid: resid[row] = x
//   out[m] = x * rsqrt(mean(x^2) + eps) * weight
// row = rows ? rows[m] : m.  With `rows`, write_resid must be 0 (a row could be
// named twice).
// ---------------------------------------------------------------------------
// delta may come as `parts` float32 partial sums, part_stride elements apart
// (a split-K product's output): they are added in order.
// Vector form: H a multiple of 4 and at most 4 * kNormGroups * blockDim.  A thread
// keeps its elements of the row in registers, and all loads of the partial sums
// are issued before the first add, so a row costs about one memory round trip.
constexpr int kNormGroups = 4;

template <typename T, typename TD>
__global__ __launch_bounds__(1024) void add_rmsnorm_vec_kernel(
    float* __restrict__ resid, const TD* __restrict__ delta, int parts, long part_stride,
    const int* __restrict__ rows, const float* __restrict__ weight, T* __restrict__ out, int H,
    float eps, int write_resid) {
  __shared__ float scratch[16];
  const int m = blockIdx.x;
  const size_t row = rows ? (size_t)rows[m] : (size_t)m;
  float* x = resid + row * H;
  const TD* dl = delta ? delta + row * H : nullptr;
  float4 xv[kNormGroups], wv[kNormGroups];
  float ss = 0.f;
  // the norm's weight is asked for with the stream, not after the rows' sums are known (a
  // memory round trip less in a kernel that is little else)
#pragma unroll
  for (int g = 0; g < kNormGroups; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    wv[g] = d < H ? *reinterpret_cast<const float4*>(weight + d) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
#pragma unroll
  for (int g = 0; g < kNormGroups; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    xv[g] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (d < H) {
      float4 v = *reinterpret_cast<const float4*>(x + d);
      if (dl) {
        int p = 0;
        for (; p + 8 <= parts; p += 8) {   // eight partial sums in flight, added in split order
          float4 q[8];
#pragma unroll
          for (int u = 0; u < 8; ++u) q[u] = Load4<TD>::at(dl + (size_t)(p + u) * part_stride + d);
#pragma unroll
          for (int u = 0; u < 8; ++u) {
            v.x += q[u].x;
            v.y += q[u].y;
            v.z += q[u].z;
            v.w += q[u].w;
          }
        }
        for (; p + 4 <= parts; p += 4) {
          const float4 a = Load4<TD>::at(dl + (size_t)p * part_stride + d);
          const float4 b = Load4<TD>::at(dl + (size_t)(p + 1) * part_stride + d);
          const float4 c = Load4<TD>::at(dl + (size_t)(p + 2) * part_stride + d);
          const float4 e = Load4<TD>::at(dl + (size_t)(p + 3) * part_stride + d);
          v.x = (((v.x + a.x) + b.x) + c.x) + e.x;
          v.y = (((v.y + a.y) + b.y) + c.y) + e.y;
          v.z = (((v.z + a.z) + b.z) + c.z) + e.z;
          v.w = (((v.w + a.w) + b.w) + c.w) + e.w;
        }
        for (; p < parts; ++p) {
          const float4 a = Load4<TD>::at(dl + (size_t)p * part_stride + d);
          v.x += a.x;
          v.y += a.y;
          v.z += a.z;
          v.w += a.w;
        }
        if (write_resid) *reinterpret_cast<float4*>(x + d) = v;
      }
      xv[g] = v;
      ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
    }
  }
  ss = block_sum(ss, scratch);
  const float rstd = rsqrtf(ss / (float)H + eps);
  T* o = out + (size_t)m * H;
#pragma unroll
  for (int g = 0; g < kNormGroups; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    if (d < H) {
      const float4 w = wv[g];
      Store4<T>::at(o + d, make_float4(xv[g].x * rstd * w.x, xv[g].y * rstd * w.y,
                                       xv[g].z * rstd * w.z, xv[g].w * rstd * w.w));
    }
  }
}

template <typename T, typename TD>
__global__ void add_rmsnorm_kernel(float* __restrict__ resid, const TD* __restrict__ delta,
                                   int parts, long part_stride, const int* __restrict__ rows,
                                   const float* __restrict__ weight, T* __restrict__ out, int H,
                                   float eps, int write_resid) {
  __shared__ float scratch[16];
  const int m = blockIdx.x;
  const size_t row = rows ? (size_t)rows[m] : (size_t)m;
  float* x = resid + row * H;
  const TD* dl = delta ? delta + row * H : nullptr;
  float ss = 0.f;
  for (int d = threadIdx.x; d < H; d += blockDim.x) {
    float v = x[d];
    if (dl) {
      for (int p = 0; p < parts; ++p) v += Elem<TD>::load(dl + (size_t)p * part_stride + d);
      if (write_resid) x[d] = v;
    }
    ss += v * v;
  }
  ss = block_sum(ss, scratch);
  const float rstd = rsqrtf(ss / (float)H + eps);
  T* o = out + (size_t)m * H;
  for (int d = threadIdx.x; d < H; d += blockDim.x) {
    float v = x[d];
    if (dl && !write_resid)
      for (int p = 0; p < parts; ++p) v += Elem<TD>::load(dl + (size_t)p * part_stride + d);
    Elem<T>::store(o + d, v * rstd * weight[d]);
  }
}

// delta_f32: delta is float32 (possibly `parts` partial sums) whatever the dtype
TK_API int tk_add_rmsnorm(int dtype, float* resid, const void* delta, int delta_f32, int parts,
                          long part_stride, const int* rows, const float* weight, void* out, int M,
                          int H, float eps, int write_resid, hipStream_t stream) {
  if (M <= 0) return 0;
  if (rows && write_resid) return -1;
  if (parts < 1 || (parts > 1 && !delta_f32 && dtype != 0)) return -1;
  // vector form when the row fits a block's registers and everything is 16-byte aligned
  // one element group per thread when rows are few (short latency chain), four when many
  int threads = 64;
  while (threads < 1024 && threads * 4 * (M >= 512 ? kNormGroups : 1) < H) threads *= 2;
  const bool vec = H % 4 == 0 && H <= threads * 4 * kNormGroups && part_stride % 4 == 0 &&
                   ((uintptr_t)resid % 16 == 0) && ((uintptr_t)delta % 16 == 0) &&
                   ((uintptr_t)weight % 16 == 0) && ((uintptr_t)out % 16 == 0);
#define TK_NORM(KERNEL, T_, TD_)                                                                 \
  KERNEL<T_, TD_><<<M, threads, 0, stream>>>(resid, (const TD_*)delta, parts, part_stride, rows, \
                                             weight, (T_*)out, H, eps, write_resid)
  if (vec) {
    if (dtype == 0) TK_NORM(add_rmsnorm_vec_kernel, float, float);
    else if (delta_f32) TK_NORM(add_rmsnorm_vec_kernel, bf16_t, float);
    else TK_NORM(add_rmsnorm_vec_kernel, bf16_t, bf16_t);
  } else {
    threads = 256;
    if (dtype == 0) TK_NORM(add_rmsnorm_kernel, float, float);
    else if (delta_f32) TK_NORM(add_rmsnorm_kernel, bf16_t, float);
    else TK_NORM(add_rmsnorm_kernel, bf16_t, bf16_t);
  }
#undef TK_NORM
  return launch_status();
}

// ---------------------------------------------------------------------------
// rotary tables: angle = float(pos) * inv_freq[j]  (one float32 product, as the
// formula is written), cos/sin [N, half]
// ---------------------------------------------------------------------------
// `amplitude` multiplies both tables (1: as they are).
__global__ void rope_tables_kernel(const int* __restrict__ positions,
                                   const float* __restrict__ inv_freq, float* __restrict__ cos_t,
                                   float* __restrict__ sin_t, int N, int half, float amplitude) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= N * half) return;
  const int n = i / half, j = i - n * half;
  const float angle = __fmul_rn((float)positions[n], inv_freq[j]);
  const float c = cosf(angle), s = sinf(angle);
  cos_t[i] = amplitude == 1.f ? c : c * amplitude;
  sin_t[i] = amplitude == 1.f ? s : s * amplitude;
}

TK_API int tk_rope_tables(const int* positions, const float* inv_freq, float* cos_t, float* sin_t,
                          int N, int half, float amplitude, hipStream_t stream) {
  const int total = N * half;
  if (total <= 0) return 0;
  rope_tables_kernel<<<(total + 255) / 256, 256, 0, stream>>>(positions, inv_freq, cos_t, sin_t, N,
                                                               half, amplitude);
  return launch_status();
}

// ---------------------------------------------------------------------------
// per-head RMSNorm of q and k, half-split rotation of the first `rot` dims,
// q written out, k and v written into the paged cache.
//
// qkv: [N, (nh + 2*nkv) * hd] (q heads, then k heads, then v heads); with
// nkv_in == 0 the input holds q heads only and nothing is stored.
// Cache pages (page_elems = nkv * hd * ps elements each):
//   K page: [nkv][hd/8][ps][8]   (8 consecutive dims of one token are adjacent,
//                                 then tokens, so lanes that hold consecutive
//                                 tokens read consecutive 16-byte pieces)
//   V page: [nkv][hd/16][ps/4][16][4]  (4 consecutive tokens of one dim adjacent,
//                                 then 16 dims, then groups of 4 tokens: the A
//                                 operand of the PV product, lane (dim, quad),
//                                 is 8 contiguous bytes and a wave reads 512
//                                 contiguous bytes)
// One wave per (token, head), four waves a block, each with an LDS row of its own.
// ---------------------------------------------------------------------------
constexpr int kMaxHeadDim = 512;
constexpr int kPairsPerBlock = 4;  // (token, head) pairs per block, one per wave

template <typename T, typename TIN>
__global__ void qknorm_rope_store_kernel(
    const TIN* __restrict__ qkv, int parts, long part_stride, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t,
    const int* __restrict__ positions, const int* __restrict__ req_of_token,
    const int* __restrict__ block_tables, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, int nh, int nkv_in, int nkv, int hd, int rot, int ps, int max_pages,
    float eps, int num_pairs) {
  __shared__ float vecs[kPairsPerBlock][kMaxHeadDim];
  const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
  const int heads = nh + 2 * nkv_in;
  const int pair = blockIdx.x * kPairsPerBlock + wave;
  if (pair >= num_pairs) return;  // nothing below synchronises across waves
  const int n = pair / heads, head = pair - n * heads;
  float* vec = vecs[wave];
  const int row_width = heads * hd;
  const TIN* src = qkv + (size_t)n * row_width + (size_t)head * hd;
  const bool is_q = head < nh;
  const bool is_k = !is_q && head < nh + nkv_in;
  const float* w = is_q ? q_weight : (is_k ? k_weight : nullptr);

  float ss = 0.f;
  for (int d = lane; d < hd; d += kWave) {
    float v = 0.f;
    for (int p = 0; p < parts; ++p) v += Elem<TIN>::load(src + (size_t)p * part_stride + d);
    vec[d] = v;
    ss += v * v;
  }
  if (is_q || is_k) {
    if (w) {
      ss = wave_sum(ss);
      const float rstd = rsqrtf(ss / (float)hd + eps);
      wave_lds_sync();
      for (int d = lane; d < hd; d += kWave) vec[d] = vec[d] * rstd * w[d];
    }
    wave_lds_sync();
    // out[j] = x[j] cos_j - x[j+half] sin_j ; out[j+half] = x[j+half] cos_j + x[j] sin_j
    const int half = rot / 2;
    float lo[kMaxHeadDim / 2 / kWave], hi[kMaxHeadDim / 2 / kWave];
    int cnt = 0;
    for (int j = lane; j < half; j += kWave, ++cnt) {
      const float c = cos_t[(size_t)n * half + j], s = sin_t[(size_t)n * half + j];
      const float a = vec[j], b = vec[j + half];
      lo[cnt] = a * c - b * s;
      hi[cnt] = b * c + a * s;
    }
    wave_lds_sync();
    cnt = 0;
    for (int j = lane; j < half; j += kWave, ++cnt) {
      vec[j] = lo[cnt];
      vec[j + half] = hi[cnt];
    }
  }
  wave_lds_sync();

  if (is_q) {
    T* dst = q_out + ((size_t)n * nh + head) * hd;
    for (int d = lane; d < hd; d += kWave) Elem<T>::store(dst + d, vec[d]);
    return;
  }
  const int pos = positions[n];
  const int page = block_tables[(size_t)req_of_token[n] * max_pages + pos / ps];
  const int off = pos % ps;
  const size_t page_elems = (size_t)nkv * hd * ps;
  if (is_k) {
    const int kvh = head - nh;
    T* base = k_cache + (size_t)page * page_elems + (size_t)kvh * hd * ps;
    for (int d = lane; d < hd; d += kWave)
      Elem<T>::store(base + ((size_t)(d >> 3) * ps + off) * 8 + (d & 7), vec[d]);
  } else {
    const int kvh = head - nh - nkv_in;
    T* base = v_cache + (size_t)page * page_elems + (size_t)kvh * hd * ps;
    for (int d = lane; d < hd; d += kWave)
      Elem<T>::store(base + ((size_t)(d >> 4) * (ps >> 2) + (off >> 2)) * 64 + (d & 15) * 4 + (off & 3), vec[d]);
  }
}

// Fast form for head sizes 64 and 128 rotated over their full width (rot == HD):
// a lane owns 8 consecutive dims of one head (one 16-byte piece), so a wave covers
// 64*8/HD (token, head) pairs; the rotation partner (dim +- HD/2) sits HD/16 lanes away, the
// sum of squares is over HD/8 neighbouring lanes.  The query heads come token by token; the
// pairs behind them are the key heads and then the value heads, each head with its tokens in
// order, so that a wave holds consecutive tokens of one head and its cache writes fall next
// to each other in the page: a key piece (8 dims of one token) beside those of the next
// tokens, and the values of four tokens that fill one quad of a page (bfloat16: exchanged
// through LDS inside the wave) as the page's own 16-byte pieces of two dims by four keys,
// where token by token they are 2-byte stores 8 bytes apart.
template <typename T, typename TIN, int HD>
__global__ __launch_bounds__(256) void qknorm_rope_store_vec_kernel(
    const TIN* __restrict__ qkv, int parts, long part_stride, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, const int* __restrict__ positions,
    const int* __restrict__ req_of_token, const int* __restrict__ block_tables,
    T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache, int N, int nh, int nkv_in,
    int nkv, int ps, int max_pages, float eps, long num_pairs) {
  constexpr int LPH = HD / 8;  // lanes per head
  __shared__ uint4 s_quad[sizeof(T) == 2 ? 256 : 1];
  const long slot = ((long)blockIdx.x * blockDim.x + threadIdx.x) / LPH;  // (token, head) pair
  if (slot >= num_pairs) return;  // whole LPH-lane groups leave together
  const int sub = threadIdx.x % LPH, d0 = sub * 8;
  const int heads = nh + 2 * nkv_in;
  const long q_pairs = (long)N * nh;
  int n, head;
  if (slot < q_pairs) {
    n = (int)((unsigned)slot / (unsigned)nh);
    head = (int)((unsigned)slot - (unsigned)n * (unsigned)nh);
  } else {
    const unsigned behind = (unsigned)(slot - q_pairs), kv = behind / (unsigned)N;
    n = (int)(behind - kv * (unsigned)N);
    head = nh + (int)kv;
  }
  const bool is_q = head < nh, is_k = !is_q && head < nh + nkv_in;
  const TIN* src = qkv + (size_t)n * heads * HD + (size_t)head * HD + d0;
  float x[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) x[e] = 0.f;
  for (int p = 0; p < parts; ++p) {
    const float4 a = Load4<TIN>::at(src + (size_t)p * part_stride);
    const float4 b = Load4<TIN>::at(src + (size_t)p * part_stride + 4);
    x[0] += a.x; x[1] += a.y; x[2] += a.z; x[3] += a.w;
    x[4] += b.x; x[5] += b.y; x[6] += b.z; x[7] += b.w;
  }
  if (is_q || is_k) {
    const float* w = is_q ? q_weight : k_weight;
    const int j0 = d0 % (HD / 2);  // index into the cos/sin row
    const float4 c0 = *reinterpret_cast<const float4*>(cos_t + (size_t)n * (HD / 2) + j0);
    const float4 c1 = *reinterpret_cast<const float4*>(cos_t + (size_t)n * (HD / 2) + j0 + 4);
    const float4 s0 = *reinterpret_cast<const float4*>(sin_t + (size_t)n * (HD / 2) + j0);
    const float4 s1 = *reinterpret_cast<const float4*>(sin_t + (size_t)n * (HD / 2) + j0 + 4);
    const float cs[8] = {c0.x, c0.y, c0.z, c0.w, c1.x, c1.y, c1.z, c1.w};
    const float sn[8] = {s0.x, s0.y, s0.z, s0.w, s1.x, s1.y, s1.z, s1.w};
    if (w) {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
#pragma unroll
      for (int m = LPH / 2; m >= 1; m >>= 1) ss += __shfl_xor(ss, m, kWave);
      const float rstd = rsqrtf(ss / (float)HD + eps);
      const float4 w0 = *reinterpret_cast<const float4*>(w + d0);
      const float4 w1 = *reinterpret_cast<const float4*>(w + d0 + 4);
      const float wv[8] = {w0.x, w0.y, w0.z, w0.w, w1.x, w1.y, w1.z, w1.w};
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = x[e] * rstd * wv[e];
    }
    // first half: x cos - partner sin; second half: x cos + partner sin
    const float sign = (d0 < HD / 2) ? -1.f : 1.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float partner = __shfl_xor(x[e], LPH / 2, kWave);
      x[e] = x[e] * cs[e] + sign * partner * sn[e];
    }
  }
  if (is_q) {
    Store4<T>::at(q_out + ((size_t)n * nh + head) * HD + d0, make_float4(x[0], x[1], x[2], x[3]));
    Store4<T>::at(q_out + ((size_t)n * nh + head) * HD + d0 + 4, make_float4(x[4], x[5], x[6], x[7]));
    return;
  }
  const int pos = positions[n];
  const int page = block_tables[(size_t)req_of_token[n] * max_pages + pos / ps];
  const int off = pos % ps;
  const size_t page_elems = (size_t)nkv * HD * ps;
  if (is_k) {
    T* base = k_cache + (size_t)page * page_elems + (size_t)(head - nh) * HD * ps;
    T* dst = base + ((size_t)sub * ps + off) * 8;  // dims d0 .. d0+7 of this token: one 8-element piece
    Store4<T>::at(dst, make_float4(x[0], x[1], x[2], x[3]));
    Store4<T>::at(dst + 4, make_float4(x[4], x[5], x[6], x[7]));
  } else {
    T* base = v_cache + (size_t)page * page_elems + (size_t)(head - nh - nkv_in) * HD * ps;
    if constexpr (sizeof(T) == 2) {
      // Four pairs in a row (a "quad" of this wave) that are four consecutive tokens of one
      // request and head and fill one quad of keys in a page?
      constexpr int QL = 4 * LPH;  // lanes of a quad
      const int lane = threadIdx.x & 63, t = (lane / LPH) & 3;
      const int first = lane / QL * QL + sub;  // the lane with these dims in the quad's first pair
      const int req = req_of_token[n];
      const bool fits = n == __shfl(n, first, kWave) + t && pos == __shfl(pos, first, kWave) + t &&
                        req == __shfl(req, first, kWave) && head == __shfl(head, first, kWave) && ((pos - t) & 3) == 0;
      const unsigned long long all = QL == 64 ? ~0ull : ((1ull << (QL & 63)) - 1) << (lane / QL * QL);
      if ((__builtin_amdgcn_ballot_w64(fits) & all) == all) {
        // every lane leaves its four dim pairs; lane t of the quad takes pair t of all four tokens
        s_quad[threadIdx.x] = make_uint4(pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3]), pack_bf16x2(x[4], x[5]),
                                         pack_bf16x2(x[6], x[7]));
        wave_lds_sync();
        const unsigned* words = reinterpret_cast<const unsigned*>(s_quad);
        const int quad0 = (int)threadIdx.x / QL * QL + sub;  // thread of the quad's first pair, these dims
        unsigned r[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) r[k] = words[(quad0 + k * LPH) * 4 + t];  // token k: dims d, d + 1
        const int d = d0 + 2 * t;
        uint4 piece;  // [dim d: keys 0..3][dim d + 1: keys 0..3]
        piece.x = (r[0] & 0xffffu) | (r[1] << 16);
        piece.y = (r[2] & 0xffffu) | (r[3] << 16);
        piece.z = (r[0] >> 16) | (r[1] & 0xffff0000u);
        piece.w = (r[2] >> 16) | (r[3] & 0xffff0000u);
        *reinterpret_cast<uint4*>(base + ((size_t)(d >> 4) * (ps >> 2) + (off >> 2)) * 64 + (d & 15) * 4) = piece;
        return;
      }
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int d = d0 + e;
      Elem<T>::store(base + ((size_t)(d >> 4) * (ps >> 2) + (off >> 2)) * 64 + (d & 15) * 4 + (off & 3), x[e]);
    }
  }
}

// in_f32: qkv is float32 (possibly `parts` partial sums, part_stride elements apart)
TK_API int tk_qknorm_rope_store(int dtype, const void* qkv, int in_f32, int parts, long part_stride,
                                const float* q_weight, const float* k_weight, const float* cos_t,
                                const float* sin_t, const int* positions, const int* req_of_token,
                                const int* block_tables, void* q_out, void* k_cache, void* v_cache,
                                int N, int nh, int nkv_in, int nkv, int hd, int rot, int ps,
                                int max_pages, float eps, hipStream_t stream) {
  if (N <= 0) return 0;
  if (hd > kMaxHeadDim || hd % 16 != 0 || ps % 4 != 0 || rot > hd || rot % 2 != 0) return -1;
  if (nkv_in != 0 && nkv_in != nkv) return -1;
  if (parts < 1 || (parts > 1 && !in_f32 && dtype != 0)) return -1;
  const long pairs = (long)N * (nh + 2 * nkv_in);
  if (pairs > 0x7fffffffL) return -1;
  if ((hd == 128 || hd == 64) && rot == hd && part_stride % 4 == 0 && (uintptr_t)qkv % 16 == 0 &&
      (uintptr_t)q_out % 16 == 0 && (uintptr_t)k_cache % 16 == 0 && (uintptr_t)cos_t % 16 == 0 &&
      (uintptr_t)sin_t % 16 == 0 && (!q_weight || (uintptr_t)q_weight % 16 == 0) &&
      (!k_weight || (uintptr_t)k_weight % 16 == 0) && (q_weight != nullptr) == (k_weight != nullptr)) {
    const long lanes = pairs * (hd / 8);
    const unsigned vgrid = (unsigned)((lanes + 255) / 256);
#define TK_QKV(T_, TIN_, HD_)                                                                     \
  qknorm_rope_store_vec_kernel<T_, TIN_, HD_><<<vgrid, 256, 0, stream>>>(                         \
      (const TIN_*)qkv, parts, part_stride, q_weight, k_weight, cos_t, sin_t, positions,          \
      req_of_token, block_tables, (T_*)q_out, (T_*)k_cache, (T_*)v_cache, N, nh, nkv_in, nkv, ps, \
      max_pages, eps, pairs)
    if (hd == 128) {
      if (dtype == 0) TK_QKV(float, float, 128);
      else if (in_f32) TK_QKV(bf16_t, float, 128);
      else TK_QKV(bf16_t, bf16_t, 128);
    } else {
      if (dtype == 0) TK_QKV(float, float, 64);
      else if (in_f32) TK_QKV(bf16_t, float, 64);
      else TK_QKV(bf16_t, bf16_t, 64);
    }
#undef TK_QKV
    return launch_status();
  }
  const unsigned grid = (unsigned)((pairs + kPairsPerBlock - 1) / kPairsPerBlock);
#define TK_QK(T_, TIN_)                                                                          \
  qknorm_rope_store_kernel<T_, TIN_><<<grid, kWave * kPairsPerBlock, 0, stream>>>(               \
      (const TIN_*)qkv, parts, part_stride, q_weight, k_weight, cos_t, sin_t, positions,         \
      req_of_token, block_tables, (T_*)q_out, (T_*)k_cache, (T_*)v_cache, nh, nkv_in, nkv, hd,   \
      rot, ps, max_pages, eps, (int)pairs)
  if (dtype == 0) TK_QK(float, float);
  else if (in_f32) TK_QK(bf16_t, float);
  else TK_QK(bf16_t, bf16_t);
#undef TK_QK
  return launch_status();
}

// ---------------------------------------------------------------------------
// out[n, i] = act(gu[n, i]) * gu[n, I + i]; act 0: silu(z) = z / (1 + exp(-z)), act 1: the tanh
// form of gelu, 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))).  act 2, a gate with clamped halves:
// with g = min(gu[n, i], limit) and u = clamp(gu[n, I + i], -limit, limit), out = g sigmoid(1.702 g) (u + 1)
// ---------------------------------------------------------------------------
__device__ __forceinline__ float gated_value(float z, float u, int act, float limit) {
  if (act == 0) return z / (1.f + expf(-z)) * u;
  if (act == 1) return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))) * u;
  const float g = fminf(z, limit);
  return g / (1.f + expf(-1.702f * g)) * (fminf(fmaxf(u, -limit), limit) + 1.f);
}

// The gate over float32 partial sums of a split product, four columns a thread: I and part_stride multiples of four.
template <typename T>
__global__ __launch_bounds__(256) void silu_mul_parts_kernel(const float* __restrict__ gu, int parts, long part_stride,
                                                             T* __restrict__ out, int I, size_t total4, int act, float limit) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total4) return;
  const int per_row = I / 4;
  const size_t n = idx / per_row;
  const int i = (int)(idx - n * per_row) * 4;
  const float* g = gu + n * 2 * I + i;
  float gv[4] = {0.f, 0.f, 0.f, 0.f}, uv[4] = {0.f, 0.f, 0.f, 0.f};
  for (int p = 0; p < parts; p += 4) {       // four partial sums of each half in flight, added in split order
    float4 a[4], b[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (p + k < parts) {
        a[k] = *reinterpret_cast<const float4*>(g + (size_t)(p + k) * part_stride);
        b[k] = *reinterpret_cast<const float4*>(g + (size_t)(p + k) * part_stride + I);
      }
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (p + k < parts) {
        gv[0] += a[k].x; gv[1] += a[k].y; gv[2] += a[k].z; gv[3] += a[k].w;
        uv[0] += b[k].x; uv[1] += b[k].y; uv[2] += b[k].z; uv[3] += b[k].w;
      }
    }
  }
  Store4<T>::at(out + n * I + i, make_float4(gated_value(gv[0], uv[0], act, limit), gated_value(gv[1], uv[1], act, limit),
                                             gated_value(gv[2], uv[2], act, limit), gated_value(gv[3], uv[3], act, limit)));
}

TK_API int tk_silu_mul_parts(int dtype, const float* gu, int parts, long part_stride, void* out, int N, int I, int act,
                             float limit, hipStream_t stream) {
  if (N <= 0 || I <= 0) return 0;
  if (act < 0 || act > 2 || parts < 1 || I % 4 != 0 || part_stride % 4 != 0 || (uintptr_t)gu % 16 != 0 || (uintptr_t)out % 16 != 0)
    return -1;
  const size_t total4 = (size_t)N * I / 4;
  const unsigned blocks = (unsigned)((total4 + 255) / 256);
  if (dtype == 0) silu_mul_parts_kernel<float><<<blocks, 256, 0, stream>>>(gu, parts, part_stride, (float*)out, I, total4, act, limit);
  else silu_mul_parts_kernel<bf16_t><<<blocks, 256, 0, stream>>>(gu, parts, part_stride, (bf16_t*)out, I, total4, act, limit);
  return launch_status();
}

template <typename T>
__global__ void silu_mul_kernel(const T* __restrict__ gu, T* __restrict__ out, int I, size_t total, int act,
                                float limit, const float* __restrict__ bias) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const size_t n = idx / I;
  const int i = (int)(idx - n * I);
  float g = Elem<T>::load(gu + n * 2 * I + i);
  float u = Elem<T>::load(gu + n * 2 * I + I + i);
  if (bias) {     // (float32 [2 I]: the gate's biases, then the up projection's)
    g += bias[i];
    u += bias[I + i];
  }
  Elem<T>::store(out + idx, gated_value(g, u, act, limit));
}

// x[n, c] += bias[c] in place (float32 bias, the sum formed in float32)
template <typename T>
__global__ void add_bias_kernel(T* __restrict__ x, const float* __restrict__ bias, int H, size_t total) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  Elem<T>::store(x + idx, Elem<T>::load(x + idx) + bias[idx % H]);
}

// 8 elements a thread (16-byte loads): I a multiple of 8, pointers 16-byte aligned
__global__ void silu_mul_bf16x8_kernel(const bf16_t* __restrict__ gu, bf16_t* __restrict__ out,
                                       int I, size_t total8, int act, float limit) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total8) return;
  const int per_row = I / 8;
  const size_t n = idx / per_row;
  const int i = (int)(idx - n * per_row) * 8;
  const uint4 g = *reinterpret_cast<const uint4*>(gu + n * 2 * I + i);
  const uint4 u = *reinterpret_cast<const uint4*>(gu + n * 2 * I + I + i);
  const uint32_t gw[4] = {g.x, g.y, g.z, g.w}, uw[4] = {u.x, u.y, u.z, u.w};
  uint32_t ow[4];
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const float g0 = __uint_as_float(gw[k] << 16), g1 = __uint_as_float(gw[k] & 0xffff0000u);
    const float u0 = __uint_as_float(uw[k] << 16), u1 = __uint_as_float(uw[k] & 0xffff0000u);
    ow[k] = pack_bf16x2(gated_value(g0, u0, act, limit), gated_value(g1, u1, act, limit));
  }
  *reinterpret_cast<uint4*>(out + n * I + i) = make_uint4(ow[0], ow[1], ow[2], ow[3]);
}

// out[n, i] = max(x[n, i], 0)^2: x is T, float32, or float32 partial sums of a split product
template <typename T>
__device__ __forceinline__ float branch_value(const void* p, int f32, int parts, long part_stride, size_t idx);

template <typename T>
__global__ void squared_relu_kernel(const void* __restrict__ x, int f32, int parts, long part_stride, T* __restrict__ out,
                                    size_t total) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const float v = fmaxf(branch_value<T>(x, f32, parts, part_stride, idx), 0.f);
  Elem<T>::store(out + idx, v * v);
}

// 8 elements a thread
__global__ void squared_relu_bf16x8_kernel(const bf16_t* __restrict__ x, bf16_t* __restrict__ out, size_t total8) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total8) return;
  const uint4 v = reinterpret_cast<const uint4*>(x)[idx];
  const uint32_t w[4] = {v.x, v.y, v.z, v.w};
  uint32_t o[4];
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const float a = fmaxf(__uint_as_float(w[k] << 16), 0.f), b = fmaxf(__uint_as_float(w[k] & 0xffff0000u), 0.f);
    o[k] = pack_bf16x2(a * a, b * b);
  }
  reinterpret_cast<uint4*>(out)[idx] = make_uint4(o[0], o[1], o[2], o[3]);
}

TK_API int tk_squared_relu(int dtype, const void* x, int f32, int parts, long part_stride, void* out, long total,
                           hipStream_t stream) {
  if (total <= 0) return 0;
  if (parts < 1 || (parts > 1 && !f32 && dtype != 0)) return -1;
  if (dtype == 1 && !f32 && parts == 1 && total % 8 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)out % 16 == 0) {
    squared_relu_bf16x8_kernel<<<(unsigned)((total / 8 + 255) / 256), 256, 0, stream>>>((const bf16_t*)x, (bf16_t*)out, (size_t)total / 8);
    return launch_status();
  }
  const unsigned blocks = (unsigned)((total + 255) / 256);
  if (dtype == 0) squared_relu_kernel<float><<<blocks, 256, 0, stream>>>(x, 1, parts, part_stride, (float*)out, (size_t)total);
  else squared_relu_kernel<bf16_t><<<blocks, 256, 0, stream>>>(x, f32, parts, part_stride, (bf16_t*)out, (size_t)total);
  return launch_status();
}

// ---------------------------------------------------------------------------
// The difference of two attention maps, per token and head: with o = a_1 - lambda a_2 over the head's vd values,
// out = o / sqrt(mean(o^2) + eps) * scale.  a: rows of 2 `heads` heads of vdp >= vd columns (map 1 and map 2 of
// head 0, then of head 1, ...); out rows: `heads` heads of vd columns, dense.  lambda is one float32 number on the
// device.  LANES neighbouring lanes take a head, four values each at a time.
// ---------------------------------------------------------------------------
template <typename T, int LANES>
__global__ __launch_bounds__(256) void map_difference_kernel(const T* __restrict__ a, const float* __restrict__ lambda,
                                                             T* __restrict__ out, int vd, int vdp, float eps, float scale,
                                                             long items) {
  constexpr int STEPS = 2;           // (16 lanes: heads of up to 128 values, 64 lanes: 512)
  const long item = (long)blockIdx.x * (256 / LANES) + threadIdx.x / LANES;
  const int sub = threadIdx.x % LANES;
  if (item >= items) return;         // (whole groups of lanes leave together)
  const float lam = *lambda;
  const T* p = a + (size_t)item * 2 * vdp;
  float o[STEPS][4];
  float ss = 0.f;
#pragma unroll
  for (int s = 0; s < STEPS; ++s) {
    const int d = (s * LANES + sub) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[s][e] = 0.f;
    if (d < vd) {
      const float4 x = Load4<T>::at(p + d), y = Load4<T>::at(p + vdp + d);
      const float xv[4] = {x.x, x.y, x.z, x.w}, yv[4] = {y.x, y.y, y.z, y.w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        if (d + e < vd) o[s][e] = xv[e] - lam * yv[e];
        ss = fmaf(o[s][e], o[s][e], ss);
      }
    }
  }
#pragma unroll
  for (int m = LANES / 2; m >= 1; m >>= 1) ss += __shfl_xor(ss, m, kWave);
  const float factor = scale / sqrtf(ss / (float)vd + eps);
  T* q = out + (size_t)item * vd;
#pragma unroll
  for (int s = 0; s < STEPS; ++s) {
    const int d = (s * LANES + sub) * 4;
    if (d >= vd) continue;
    if (vd % 4 == 0) {
      Store4<T>::at(q + d, make_float4(o[s][0] * factor, o[s][1] * factor, o[s][2] * factor, o[s][3] * factor));
    } else {
      for (int e = 0; e < 4 && d + e < vd; ++e) Elem<T>::store(q + d + e, o[s][e] * factor);
    }
  }
}

TK_API int tk_map_difference(int dtype, const void* a, const float* lambda, void* out, int N, int heads, int vd, int vdp,
                             float eps, float scale, hipStream_t stream) {
  if (N <= 0) return 0;
  if (heads < 1 || vd < 1 || vdp < vd || vdp % 16 != 0 || vdp > 512 || lambda == nullptr) return -1;
  if ((uintptr_t)a % 16 != 0 || (uintptr_t)out % 16 != 0) return -1;
  const long items = (long)N * heads;
#define TK_MD(T_, LANES_)                                                                                       \
  map_difference_kernel<T_, LANES_><<<(unsigned)((items + 256 / LANES_ - 1) / (256 / LANES_)), 256, 0, stream>>>( \
      (const T_*)a, lambda, (T_*)out, vd, vdp, eps, scale, items)
  if (vd <= 128) {
    if (dtype == 0) TK_MD(float, 16);
    else TK_MD(bf16_t, 16);
  } else {
    if (dtype == 0) TK_MD(float, 64);
    else TK_MD(bf16_t, 64);
  }
#undef TK_MD
  return launch_status();
}

TK_API int tk_add_bias(int dtype, void* x, const float* bias, int N, int H, hipStream_t stream) {
  if (N <= 0 || H <= 0) return 0;
  const size_t total = (size_t)N * H;
  const unsigned blocks = (unsigned)((total + 255) / 256);
  if (dtype == 0) add_bias_kernel<float><<<blocks, 256, 0, stream>>>((float*)x, bias, H, total);
  else add_bias_kernel<bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)x, bias, H, total);
  return launch_status();
}

// bias: null, or float32 [2 I] added to the gate's and the up projection's halves before the activation
TK_API int tk_silu_mul(int dtype, const void* gu, void* out, int N, int I, int act, float limit, const float* bias,
                       hipStream_t stream) {
  if (N <= 0 || I <= 0) return 0;
  if (act < 0 || act > 2) return -1;
  const size_t total = (size_t)N * I;
  if (bias == nullptr && dtype == 1 && I % 8 == 0 && (uintptr_t)gu % 16 == 0 && (uintptr_t)out % 16 == 0) {
    const size_t total8 = total / 8;
    silu_mul_bf16x8_kernel<<<(unsigned)((total8 + 255) / 256), 256, 0, stream>>>(
        (const bf16_t*)gu, (bf16_t*)out, I, total8, act, limit);
    return launch_status();
  }
  const unsigned blocks = (unsigned)((total + 255) / 256);
  if (dtype == 0)
    silu_mul_kernel<float><<<blocks, 256, 0, stream>>>((const float*)gu, (float*)out, I, total, act, limit, bias);
  else
    silu_mul_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)gu, (bf16_t*)out, I, total, act, limit, bias);
  return launch_status();
}

// ---------------------------------------------------------------------------
// out[n, c] = scale[c] * (wa * a[n, c] + wb * b[n, c]), float32: the sum of a layer's parallel
// branches, each with its weight, times a per-coordinate layer scale.  a and b are each T,
// float32, or float32 partial sums of a split product; b may be absent.
template <typename T>
__device__ __forceinline__ float branch_value(const void* p, int f32, int parts, long part_stride, size_t idx) {
  if (!f32) return Elem<T>::load(reinterpret_cast<const T*>(p) + idx);
  const float* f = reinterpret_cast<const float*>(p);
  float s = f[idx];
  for (int i = 1; i < parts; ++i) s += f[idx + (size_t)i * part_stride];
  return s;
}

template <typename T>
__global__ void scaled_sum_kernel(const void* __restrict__ a, int a_f32, int a_parts, long a_stride, float wa,
                                  const void* __restrict__ b, int b_f32, int b_parts, long b_stride, float wb,
                                  const float* __restrict__ scale, float* __restrict__ out, int H, size_t total) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  float v = wa * branch_value<T>(a, a_f32, a_parts, a_stride, idx);
  if (b != nullptr) v = fmaf(wb, branch_value<T>(b, b_f32, b_parts, b_stride, idx), v);
  if (scale != nullptr) v *= scale[idx % H];
  out[idx] = v;
}

// four consecutive columns a thread: H a multiple of 4 (every row then starts on a border of four)
template <typename T>
__device__ __forceinline__ float4 branch_four(const void* p, int f32, int parts, long part_stride, size_t idx) {
  if (!f32) return Load4<T>::at(reinterpret_cast<const T*>(p) + idx);
  const float* f = reinterpret_cast<const float*>(p) + idx;
  float4 s = *reinterpret_cast<const float4*>(f);
  for (int i = 1; i < parts; ++i) {
    const float4 a = *reinterpret_cast<const float4*>(f + (size_t)i * part_stride);
    s.x += a.x; s.y += a.y; s.z += a.z; s.w += a.w;
  }
  return s;
}

template <typename T>
__global__ void scaled_sum_four_kernel(const void* __restrict__ a, int a_f32, int a_parts, long a_stride, float wa,
                                       const void* __restrict__ b, int b_f32, int b_parts, long b_stride, float wb,
                                       const float* __restrict__ scale, float* __restrict__ out, int H, size_t total4) {
  const size_t i4 = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i4 >= total4) return;
  const size_t idx = i4 * 4;
  const float4 x = branch_four<T>(a, a_f32, a_parts, a_stride, idx);
  float4 v = make_float4(wa * x.x, wa * x.y, wa * x.z, wa * x.w);
  if (b != nullptr) {
    const float4 y = branch_four<T>(b, b_f32, b_parts, b_stride, idx);
    v = make_float4(fmaf(wb, y.x, v.x), fmaf(wb, y.y, v.y), fmaf(wb, y.z, v.z), fmaf(wb, y.w, v.w));
  }
  if (scale != nullptr) {
    const float4 g = *reinterpret_cast<const float4*>(scale + idx % H);
    v = make_float4(v.x * g.x, v.y * g.y, v.z * g.z, v.w * g.w);
  }
  *reinterpret_cast<float4*>(out + idx) = v;
}

TK_API int tk_scaled_sum(int dtype, const void* a, int a_f32, int a_parts, long a_stride, float wa,
                         const void* b, int b_f32, int b_parts, long b_stride, float wb, const float* scale,
                         float* out, int N, int H, hipStream_t stream) {
  if (N <= 0 || H <= 0) return 0;
  const size_t total = (size_t)N * H;
  if (H % 4 == 0 && a_stride % 4 == 0 && b_stride % 4 == 0) {
    const size_t total4 = total / 4;
    const unsigned blocks4 = (unsigned)((total4 + 255) / 256);
    if (dtype == 0)
      scaled_sum_four_kernel<float><<<blocks4, 256, 0, stream>>>(a, a_f32, a_parts, a_stride, wa, b, b_f32, b_parts,
                                                                 b_stride, wb, scale, out, H, total4);
    else
      scaled_sum_four_kernel<bf16_t><<<blocks4, 256, 0, stream>>>(a, a_f32, a_parts, a_stride, wa, b, b_f32, b_parts,
                                                                  b_stride, wb, scale, out, H, total4);
    return launch_status();
  }
  const unsigned blocks = (unsigned)((total + 255) / 256);
  if (dtype == 0)
    scaled_sum_kernel<float><<<blocks, 256, 0, stream>>>(a, a_f32, a_parts, a_stride, wa, b, b_f32, b_parts,
                                                         b_stride, wb, scale, out, H, total);
  else
    scaled_sum_kernel<bf16_t><<<blocks, 256, 0, stream>>>(a, a_f32, a_parts, a_stride, wa, b, b_f32, b_parts,
                                                          b_stride, wb, scale, out, H, total);
  return launch_status();
}

// ---------------------------------------------------------------------------
// Residual add of up to three parallel branches + norm over rows of width H.
//   x = resid[row] + scale * (a[row] + b[row] + c[row] + bias);  if write_resid: resid[row] = x
//   center: out[m] = (x - mean(x)) * rsqrt(mean((x - mean(x))^2) + eps) * weight   (a layer norm without a bias)
//   else:   out[m] = x * rsqrt(mean(x^2) + eps) * weight
// A branch is T, float32, or float32 partial sums (added in order); each may be absent; b and c may have a
// float32 weight per row (a token's gate on a whole branch).  Absent may be the
// bias too (float32 [H], one row for all).  The branches' sum is formed first, in float32, and
// added to the stream once.  weight2 / out2 (both or neither): the same normalised row times a
// second weight, for a layer whose two sub-layers each have a norm of their own over the same stream.
// ---------------------------------------------------------------------------
struct NormBranch {
  const void* p;
  int f32;
  int parts;
  long stride;
  const float* row_weight;   // null, or [rows]: the branch's row times this number (add_norm2 only)
};

struct NormAdds {
  NormBranch a, b, c;
  const float* bias;
  float scale;
  __device__ __forceinline__ bool any() const { return a.p || b.p || c.p || bias; }
};

template <typename T>
__device__ __forceinline__ float4 branch_four(const NormBranch& b, size_t idx) {
  if (!b.f32) return Load4<T>::at(reinterpret_cast<const T*>(b.p) + idx);
  const float* f = reinterpret_cast<const float*>(b.p) + idx;
  float4 s = *reinterpret_cast<const float4*>(f);
  for (int i = 1; i < b.parts; i += 8) {      // eight partial sums in flight, added in split order
    float4 q[8];
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (i + u < b.parts) q[u] = *reinterpret_cast<const float4*>(f + (size_t)(i + u) * b.stride);
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      if (i + u < b.parts) {
        s.x += q[u].x; s.y += q[u].y; s.z += q[u].z; s.w += q[u].w;
      }
    }
  }
  return s;
}

// scale * (a + b + c + bias) at four consecutive columns from d of a row that starts at `at`
template <typename T>
__device__ __forceinline__ float4 adds_four(const NormAdds& n, size_t row, size_t at, int d) {
  float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
  if (n.a.p) s = branch_four<T>(n.a, at + d);
  if (n.b.p) {
    const float4 t = branch_four<T>(n.b, at + d);
    const float w = n.b.row_weight ? n.b.row_weight[row] : 1.f;
    s.x = fmaf(w, t.x, s.x); s.y = fmaf(w, t.y, s.y); s.z = fmaf(w, t.z, s.z); s.w = fmaf(w, t.w, s.w);
  }
  if (n.c.p) {
    const float4 t = branch_four<T>(n.c, at + d);
    const float w = n.c.row_weight ? n.c.row_weight[row] : 1.f;
    s.x = fmaf(w, t.x, s.x); s.y = fmaf(w, t.y, s.y); s.z = fmaf(w, t.z, s.z); s.w = fmaf(w, t.w, s.w);
  }
  if (n.bias) {
    const float4 t = *reinterpret_cast<const float4*>(n.bias + d);
    s.x += t.x; s.y += t.y; s.z += t.z; s.w += t.w;
  }
  if (n.scale != 1.f) { s.x *= n.scale; s.y *= n.scale; s.z *= n.scale; s.w *= n.scale; }
  return s;
}

template <typename T>
__device__ __forceinline__ float adds_value(const NormAdds& n, size_t row, size_t at, int d) {
  float s = 0.f;
  if (n.a.p) s = branch_value<T>(n.a.p, n.a.f32, n.a.parts, n.a.stride, at + d);
  if (n.b.p) s = fmaf(n.b.row_weight ? n.b.row_weight[row] : 1.f, branch_value<T>(n.b.p, n.b.f32, n.b.parts, n.b.stride, at + d), s);
  if (n.c.p) s = fmaf(n.c.row_weight ? n.c.row_weight[row] : 1.f, branch_value<T>(n.c.p, n.c.f32, n.c.parts, n.c.stride, at + d), s);
  if (n.bias) s += n.bias[d];
  return n.scale != 1.f ? s * n.scale : s;
}

// Vector form: a thread keeps up to kNormGroups pieces of four elements of the row in registers.
template <typename T>
__global__ __launch_bounds__(1024) void add_norm2_vec_kernel(
    float* __restrict__ resid, NormAdds adds, const int* __restrict__ rows,
    const float* __restrict__ weight, T* __restrict__ out, const float* __restrict__ weight2, T* __restrict__ out2,
    int H, float eps, int write_resid, int center) {
  __shared__ float scratch[16];
  const int m = blockIdx.x;
  const size_t row = rows ? (size_t)rows[m] : (size_t)m;
  float* x = resid + row * H;
  float4 xv[kNormGroups], wv[kNormGroups];
  float sum = 0.f;
  const bool adding = adds.any();
#pragma unroll
  for (int g = 0; g < kNormGroups; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    wv[g] = d < H ? *reinterpret_cast<const float4*>(weight + d) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
#pragma unroll
  for (int g = 0; g < kNormGroups; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    xv[g] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (d < H) {
      float4 v = *reinterpret_cast<const float4*>(x + d);
      if (adding) {
        const float4 s = adds_four<T>(adds, row, row * H, d);
        v.x += s.x; v.y += s.y; v.z += s.z; v.w += s.w;
        if (write_resid) *reinterpret_cast<float4*>(x + d) = v;
      }
      xv[g] = v;
      sum += (v.x + v.y) + (v.z + v.w);
    }
  }
  float mean = 0.f;
  if (center) mean = block_sum(sum, scratch) / (float)H;
  float ss = 0.f;
#pragma unroll
  for (int g = 0; g < kNormGroups; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    if (d < H) {
      xv[g].x -= mean; xv[g].y -= mean; xv[g].z -= mean; xv[g].w -= mean;
      ss += xv[g].x * xv[g].x + xv[g].y * xv[g].y + xv[g].z * xv[g].z + xv[g].w * xv[g].w;
    }
  }
  ss = block_sum(ss, scratch);
  const float rstd = 1.f / sqrtf(ss / (float)H + eps);
  T* o = out + (size_t)m * H;
#pragma unroll
  for (int g = 0; g < kNormGroups; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    if (d < H) {
      const float4 w = wv[g];
      Store4<T>::at(o + d, make_float4(xv[g].x * rstd * w.x, xv[g].y * rstd * w.y,
                                       xv[g].z * rstd * w.z, xv[g].w * rstd * w.w));
      if (out2) {
        const float4 w2 = *reinterpret_cast<const float4*>(weight2 + d);
        Store4<T>::at(out2 + (size_t)m * H + d, make_float4(xv[g].x * rstd * w2.x, xv[g].y * rstd * w2.y,
                                                            xv[g].z * rstd * w2.z, xv[g].w * rstd * w2.w));
      }
    }
  }
}

// Any width and alignment: the row is walked three times (mean, variance, output).
template <typename T>
__global__ void add_norm2_kernel(float* __restrict__ resid, NormAdds adds,
                                 const int* __restrict__ rows, const float* __restrict__ weight,
                                 T* __restrict__ out, const float* __restrict__ weight2, T* __restrict__ out2,
                                 int H, float eps, int write_resid, int center) {
  __shared__ float scratch[16];
  const int m = blockIdx.x;
  const size_t row = rows ? (size_t)rows[m] : (size_t)m;
  float* x = resid + row * H;
  const bool adding = adds.any();
  float sum = 0.f;
  for (int d = threadIdx.x; d < H; d += blockDim.x) {
    float v = x[d];
    if (adding) {
      v += adds_value<T>(adds, row, row * H, d);
      if (write_resid) x[d] = v;      // (the passes below then read the sum back)
    }
    sum += v;
  }
  const bool again = adding && !write_resid;    // the sum is not in the stream: it is formed again
  float mean = 0.f;
  if (center) mean = block_sum(sum, scratch) / (float)H;
  float ss = 0.f;
  for (int d = threadIdx.x; d < H; d += blockDim.x) {
    float v = x[d];
    if (again) v += adds_value<T>(adds, row, row * H, d);
    ss += (v - mean) * (v - mean);
  }
  ss = block_sum(ss, scratch);
  const float rstd = 1.f / sqrtf(ss / (float)H + eps);
  T* o = out + (size_t)m * H;
  for (int d = threadIdx.x; d < H; d += blockDim.x) {
    float v = x[d];
    if (again) v += adds_value<T>(adds, row, row * H, d);
    Elem<T>::store(o + d, (v - mean) * rstd * weight[d]);
    if (out2) Elem<T>::store(out2 + (size_t)m * H + d, (v - mean) * rstd * weight2[d]);
  }
}

TK_API int tk_add_norm2(int dtype, float* resid, const void* a, int a_f32, int a_parts, long a_stride,
                        const void* b, int b_f32, int b_parts, long b_stride, const void* c, int c_f32, int c_parts,
                        long c_stride, const float* b_rows, const float* c_rows, const float* bias, float scale,
                        const int* rows, const float* weight, void* out, const float* weight2, void* out2, int M, int H, float eps,
                        int write_resid, int center, hipStream_t stream) {
  if (M <= 0) return 0;
  if (rows && write_resid) return -1;
  if ((weight2 == nullptr) != (out2 == nullptr)) return -1;
  if (a_parts < 1 || b_parts < 1 || c_parts < 1 || (a_parts > 1 && !a_f32) || (b_parts > 1 && !b_f32) || (c_parts > 1 && !c_f32)) return -1;
  const NormAdds adds{{a, a_f32 || dtype == 0, a_parts, a_stride, nullptr}, {b, b_f32 || dtype == 0, b_parts, b_stride, b_rows},
                      {c, c_f32 || dtype == 0, c_parts, c_stride, c_rows}, bias, scale};
  int threads = 64;
  while (threads < 1024 && threads * 4 * (M >= 512 ? kNormGroups : 1) < H) threads *= 2;
  const bool vec = H % 4 == 0 && H <= threads * 4 * kNormGroups && a_stride % 4 == 0 && b_stride % 4 == 0 && c_stride % 4 == 0 &&
                   ((uintptr_t)resid % 16 == 0) && ((uintptr_t)a % 16 == 0) && ((uintptr_t)b % 16 == 0) &&
                   ((uintptr_t)c % 16 == 0) && ((uintptr_t)bias % 16 == 0) && ((uintptr_t)weight % 16 == 0) &&
                   ((uintptr_t)out % 16 == 0) && ((uintptr_t)weight2 % 16 == 0) && ((uintptr_t)out2 % 16 == 0);
  if (vec) {
    if (dtype == 0) add_norm2_vec_kernel<float><<<M, threads, 0, stream>>>(resid, adds, rows, weight, (float*)out, weight2, (float*)out2, H, eps, write_resid, center);
    else add_norm2_vec_kernel<bf16_t><<<M, threads, 0, stream>>>(resid, adds, rows, weight, (bf16_t*)out, weight2, (bf16_t*)out2, H, eps, write_resid, center);
  } else {
    if (dtype == 0) add_norm2_kernel<float><<<M, 256, 0, stream>>>(resid, adds, rows, weight, (float*)out, weight2, (float*)out2, H, eps, write_resid, center);
    else add_norm2_kernel<bf16_t><<<M, 256, 0, stream>>>(resid, adds, rows, weight, (bf16_t*)out, weight2, (bf16_t*)out2, H, eps, write_resid, center);
  }
  return launch_status();
}

// ---------------------------------------------------------------------------
// Residual add of a sub-layer's NORMED output (a layer whose norm stands behind its sub-layers).
//   A = a[row] + bias, B = b[row];  with a gain of its own each is divided by its root mean square first: A <- A / rms(A) gain_a
//   m = wa A + wb B;  with `gain`: m <- m / rms(m) gain
//   x = resid[row] + m;  if write_resid: resid[row] = x
//   out[m] = weight ? x * rsqrt(mean(x^2) + eps_out) * weight : x
// All of it in float32, one rounding into out (which may be absent: the stream itself is read).  A branch is T,
// float32, or float32 partial sums (added in order); b, the bias, every gain and the weight may be absent, and so
// may both branches (m = 0).  A block a row.
// ---------------------------------------------------------------------------
struct NormedAdds {
  NormBranch a, b;
  const float *bias, *gain_a, *gain_b, *gain;
  float wa, wb, eps;
};

// sums of two values over a block (scratch: 32 floats)
__device__ __forceinline__ void block_sum2(float& u, float& v, float* scratch) {
  u = wave_sum(u);
  v = wave_sum(v);
  const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave, nwaves = (blockDim.x + kWave - 1) / kWave;
  __syncthreads();
  if (lane == 0) {
    scratch[wave] = u;
    scratch[16 + wave] = v;
  }
  __syncthreads();
  u = v = 0.f;
  for (int i = 0; i < nwaves; ++i) {
    u += scratch[i];
    v += scratch[16 + i];
  }
}

__device__ __forceinline__ float square_sum(const float4& v) { return v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w; }
__device__ __forceinline__ void scale_by(float4& v, float s, const float* w) {
  const float4 g = *reinterpret_cast<const float4*>(w);
  v = make_float4(v.x * s * g.x, v.y * s * g.y, v.z * s * g.z, v.w * s * g.w);
}

// Vector form: a thread keeps up to GROUPS pieces of four elements of the row in registers.
template <typename T, int GROUPS>
__global__ __launch_bounds__(1024) void add_normed_vec_kernel(
    float* __restrict__ resid, NormedAdds n, const int* __restrict__ rows, const float* __restrict__ weight,
    T* __restrict__ out, int H, float eps_out, int write_resid) {
  __shared__ float scratch[32];
  const int m = blockIdx.x;
  const size_t row = rows ? (size_t)rows[m] : (size_t)m;
  float* x = resid + row * H;
  float4 av[GROUPS], bv[GROUPS], xv[GROUPS];
  float sa = 0.f, sb = 0.f;
#pragma unroll
  for (int g = 0; g < GROUPS; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    av[g] = bv[g] = xv[g] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (d < H) {
      xv[g] = *reinterpret_cast<const float4*>(x + d);
      if (n.a.p) av[g] = branch_four<T>(n.a, row * H + d);
      if (n.b.p) bv[g] = branch_four<T>(n.b, row * H + d);
      if (n.bias) {
        const float4 t = *reinterpret_cast<const float4*>(n.bias + d);
        av[g].x += t.x; av[g].y += t.y; av[g].z += t.z; av[g].w += t.w;
      }
      sa += square_sum(av[g]);
      sb += square_sum(bv[g]);
    }
  }
  float4 gv[GROUPS];      // (the last gain is asked for with the rows, not behind the sums)
#pragma unroll
  for (int g = 0; g < GROUPS; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    gv[g] = n.gain && d < H ? *reinterpret_cast<const float4*>(n.gain + d) : make_float4(1.f, 1.f, 1.f, 1.f);
  }
  if (n.gain_a || n.gain_b) {      // (every thread of the block alike)
    block_sum2(sa, sb, scratch);
    const float ra = 1.f / sqrtf(sa / (float)H + n.eps), rb = 1.f / sqrtf(sb / (float)H + n.eps);
#pragma unroll
    for (int g = 0; g < GROUPS; ++g) {
      const int d = (g * blockDim.x + threadIdx.x) * 4;
      if (d < H) {
        if (n.gain_a) scale_by(av[g], ra, n.gain_a + d);
        if (n.gain_b) scale_by(bv[g], rb, n.gain_b + d);
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int g = 0; g < GROUPS; ++g) {
    av[g] = make_float4(n.wa * av[g].x + n.wb * bv[g].x, n.wa * av[g].y + n.wb * bv[g].y,
                        n.wa * av[g].z + n.wb * bv[g].z, n.wa * av[g].w + n.wb * bv[g].w);
    ss += square_sum(av[g]);
  }
  float rstd = 1.f;
  if (n.gain) rstd = 1.f / sqrtf(block_sum(ss, scratch) / (float)H + n.eps);
  ss = 0.f;
#pragma unroll
  for (int g = 0; g < GROUPS; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    if (d < H) {
      if (n.gain) av[g] = make_float4(av[g].x * rstd * gv[g].x, av[g].y * rstd * gv[g].y, av[g].z * rstd * gv[g].z, av[g].w * rstd * gv[g].w);
      xv[g].x += av[g].x; xv[g].y += av[g].y; xv[g].z += av[g].z; xv[g].w += av[g].w;
      if (write_resid) *reinterpret_cast<float4*>(x + d) = xv[g];
      ss += square_sum(xv[g]);
    }
  }
  if (!out) return;
  if (weight) rstd = 1.f / sqrtf(block_sum(ss, scratch) / (float)H + eps_out);
  T* o = out + (size_t)m * H;
#pragma unroll
  for (int g = 0; g < GROUPS; ++g) {
    const int d = (g * blockDim.x + threadIdx.x) * 4;
    if (d < H) {
      if (weight) scale_by(xv[g], rstd, weight + d);
      Store4<T>::at(o + d, xv[g]);
    }
  }
}

// Any width and alignment: the row's m and x wait in LDS (H floats) between the passes.
template <typename T>
__global__ __launch_bounds__(256) void add_normed_kernel(
    float* __restrict__ resid, NormedAdds n, const int* __restrict__ rows, const float* __restrict__ weight,
    T* __restrict__ out, int H, float eps_out, int write_resid) {
  __shared__ float scratch[32];
  extern __shared__ float held[];
  const int m = blockIdx.x;
  const size_t row = rows ? (size_t)rows[m] : (size_t)m;
  float* x = resid + row * H;
  auto first = [&](int d) {
    return (n.a.p ? branch_value<T>(n.a.p, n.a.f32, n.a.parts, n.a.stride, row * H + d) : 0.f) + (n.bias ? n.bias[d] : 0.f);
  };
  auto second = [&](int d) { return n.b.p ? branch_value<T>(n.b.p, n.b.f32, n.b.parts, n.b.stride, row * H + d) : 0.f; };
  float ra = 1.f, rb = 1.f;
  if (n.gain_a || n.gain_b) {
    float sa = 0.f, sb = 0.f;
    for (int d = threadIdx.x; d < H; d += blockDim.x) {
      const float a = first(d), b = second(d);
      sa = fmaf(a, a, sa);
      sb = fmaf(b, b, sb);
    }
    block_sum2(sa, sb, scratch);
    ra = 1.f / sqrtf(sa / (float)H + n.eps);
    rb = 1.f / sqrtf(sb / (float)H + n.eps);
  }
  float ss = 0.f;
  for (int d = threadIdx.x; d < H; d += blockDim.x) {      // (a thread reads back only what it wrote itself)
    const float a = n.gain_a ? first(d) * ra * n.gain_a[d] : first(d), b = n.gain_b ? second(d) * rb * n.gain_b[d] : second(d);
    const float v = n.wa * a + n.wb * b;
    held[d] = v;
    ss = fmaf(v, v, ss);
  }
  float rstd = 1.f;
  if (n.gain) rstd = 1.f / sqrtf(block_sum(ss, scratch) / (float)H + n.eps);
  ss = 0.f;
  for (int d = threadIdx.x; d < H; d += blockDim.x) {
    const float v = x[d] + (n.gain ? held[d] * rstd * n.gain[d] : held[d]);
    if (write_resid) x[d] = v;
    held[d] = v;
    ss = fmaf(v, v, ss);
  }
  if (!out) return;
  if (weight) rstd = 1.f / sqrtf(block_sum(ss, scratch) / (float)H + eps_out);
  for (int d = threadIdx.x; d < H; d += blockDim.x)
    Elem<T>::store(out + (size_t)m * H + d, weight ? held[d] * rstd * weight[d] : held[d]);
}

TK_API int tk_add_normed(int dtype, float* resid, const void* a, int a_f32, int a_parts, long a_stride, const float* bias,
                         const float* gain_a, float wa, const void* b, int b_f32, int b_parts, long b_stride,
                         const float* gain_b, float wb, const float* gain, float eps, const int* rows,
                         const float* weight, float eps_out, void* out, int M, int H, int write_resid, hipStream_t stream) {
  if (M <= 0) return 0;
  if (rows && write_resid) return -1;
  if (a_parts < 1 || b_parts < 1 || (a_parts > 1 && !a_f32) || (b_parts > 1 && !b_f32) || (weight && !out)) return -1;
  const NormedAdds adds{{a, a_f32 || dtype == 0, a_parts, a_stride}, {b, b_f32 || dtype == 0, b_parts, b_stride},
                        bias, gain_a, gain_b, gain, wa, wb, eps};
  int threads = 64;
  while (threads < 1024 && threads * 4 * (M >= 512 ? kNormGroups : 1) < H) threads *= 2;
  const bool vec = H % 4 == 0 && H <= threads * 4 * kNormGroups && a_stride % 4 == 0 && b_stride % 4 == 0 &&
                   (uintptr_t)resid % 16 == 0 && (uintptr_t)a % 16 == 0 && (uintptr_t)b % 16 == 0 && (uintptr_t)bias % 16 == 0 &&
                   (uintptr_t)gain_a % 16 == 0 && (uintptr_t)gain_b % 16 == 0 && (uintptr_t)gain % 16 == 0 &&
                   (uintptr_t)weight % 16 == 0 && (uintptr_t)out % 16 == 0;
#define TK_AN(KERNEL, T_, THREADS_, LDS_) \
  KERNEL<<<M, THREADS_, LDS_, stream>>>(resid, adds, rows, weight, (T_*)out, H, eps_out, write_resid)
  if (vec) {
    const bool one = threads * 4 >= H;
    if (dtype == 0) {
      if (one) TK_AN((add_normed_vec_kernel<float, 1>), float, threads, 0);
      else TK_AN((add_normed_vec_kernel<float, kNormGroups>), float, threads, 0);
    } else {
      if (one) TK_AN((add_normed_vec_kernel<bf16_t, 1>), bf16_t, threads, 0);
      else TK_AN((add_normed_vec_kernel<bf16_t, kNormGroups>), bf16_t, threads, 0);
    }
    return launch_status();
  }
  const size_t lds = (size_t)H * 4;
  if (lds > 60 * 1024) return -1;
  if (dtype == 0) TK_AN((add_normed_kernel<float>), float, 256, lds);
  else TK_AN((add_normed_kernel<bf16_t>), bf16_t, 256, lds);
#undef TK_AN
  return launch_status();
}

// ---------------------------------------------------------------------------
// x[n, head, d] *= sigmoid(gate[n, head * vd + d]) in place: the gate behind attention (per_head: the gate holds
// one number a head instead, gate[n, head]).  x rows hold `heads`
// heads of vdp >= vd columns (those behind vd stay as they are); gate rows are ld long and start at column col0,
// in T, float32, or float32 partial sums.
// ---------------------------------------------------------------------------
template <typename T>
__global__ void sigmoid_gate_kernel(T* __restrict__ x, const void* __restrict__ gate, int f32, int parts, long part_stride,
                                    long ld, int col0, int width, int vd, int vdp, int per_head, size_t total) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const size_t n = idx / width;
  const int c = (int)(idx - n * width);
  const int head = c / vd, d = c - head * vd;
  const float g = branch_value<T>(gate, f32, parts, part_stride, n * ld + col0 + (per_head ? head : c));
  T* at = x + n * ((size_t)(width / vd) * vdp) + (size_t)head * vdp + d;
  Elem<T>::store(at, Elem<T>::load(at) / (1.f + expf(-g)));
}

// four neighbouring columns a thread: vd and vdp multiples of four, and with a gate per column ld, col0 and
// part_stride too
template <typename T>
__global__ void sigmoid_gate_four_kernel(T* __restrict__ x, NormBranch gate, long ld, int col0, int width, int vd, int vdp,
                                         int per_head, size_t total4) {
  const size_t i4 = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i4 >= total4) return;
  const int quads = width / 4;
  const size_t n = i4 / quads;
  const int c = (int)(i4 - n * quads) * 4;
  const int head = c / vd, d = c - head * vd;
  float4 g;
  if (per_head) {
    g.x = branch_value<T>(gate.p, gate.f32, gate.parts, gate.stride, n * ld + col0 + head);
    g.y = g.z = g.w = g.x;
  } else {
    g = branch_four<T>(gate, n * ld + col0 + c);
  }
  T* at = x + n * ((size_t)(width / vd) * vdp) + (size_t)head * vdp + d;
  const float4 v = Load4<T>::at(at);
  Store4<T>::at(at, make_float4(v.x / (1.f + expf(-g.x)), v.y / (1.f + expf(-g.y)), v.z / (1.f + expf(-g.z)), v.w / (1.f + expf(-g.w))));
}

TK_API int tk_sigmoid_gate(int dtype, void* x, const void* gate, int f32, int parts, long part_stride, long ld, int col0,
                           int N, int heads, int vd, int vdp, int per_head, hipStream_t stream) {
  if (N <= 0) return 0;
  if (heads < 1 || vd < 1 || vdp < vd || parts < 1 || (parts > 1 && !f32 && dtype != 0) || col0 < 0 ||
      ld < (long)col0 + (long)heads * (per_head ? 1 : vd))
    return -1;
  const size_t total = (size_t)N * heads * vd;
  const bool gate_wide = ld % 4 == 0 && col0 % 4 == 0 && part_stride % 4 == 0 && (uintptr_t)gate % 16 == 0;
  if (vd % 4 == 0 && vdp % 4 == 0 && (per_head || gate_wide) && (uintptr_t)x % 16 == 0) {
    const unsigned quads = (unsigned)((total / 4 + 255) / 256);
    const NormBranch g{gate, f32 || dtype == 0, parts, part_stride, nullptr};
    if (dtype == 0) sigmoid_gate_four_kernel<float><<<quads, 256, 0, stream>>>((float*)x, g, ld, col0, heads * vd, vd, vdp, per_head, total / 4);
    else sigmoid_gate_four_kernel<bf16_t><<<quads, 256, 0, stream>>>((bf16_t*)x, g, ld, col0, heads * vd, vd, vdp, per_head, total / 4);
    return launch_status();
  }
  const unsigned blocks = (unsigned)((total + 255) / 256);
  if (dtype == 0)
    sigmoid_gate_kernel<float><<<blocks, 256, 0, stream>>>((float*)x, gate, 1, parts, part_stride, ld, col0, heads * vd, vd, vdp, per_head, total);
  else
    sigmoid_gate_kernel<bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)x, gate, f32, parts, part_stride, ld, col0, heads * vd, vd, vdp, per_head, total);
  return launch_status();
}

// ---------------------------------------------------------------------------
// Rotation of the first `rot` dims of q and k (half-split pairs, dim j with j + rot/2, or
// `interleaved` pairs, dim 2j with 2j + 1), THEN (unit) each head of q and k divided by
// its root mean square over all hd dims (times a weight per dim, if one is given), q written
// out, k and v written into the paged cache.  Keys and values may differ in size:
// qkv: [N, nh * hd + nkv_in * hd + nkv_in * vd] (q heads, k heads, v heads); with nkv_in == 0
// the input holds q heads only and nothing is stored.  Cache pages as above, the value page
// with a size of its own: K page [nkv][hdp/8][ps][8], V page [nkv][vdp/16][ps/4][16][4], where
// hdp >= hd and vdp >= vd are the sizes the pages and q_out are laid out for (hd rounded up to 8,
// vd to 16): the channels behind hd are written as zeros into q_out and never written in the
// pages (which start as zeros), so they add nothing to a score or an output.
// norm_first: the norm comes before the rotation instead.  bias (float32, one for every q, k and v column that
// the input holds) is added before anything else.  Input rows are in_ld long (columns behind the heads are not read).
// Values may be mixed with those another layer made for the same tokens (v_keep, float32
// [N, nkv * vd]): v_mode 1 leaves this layer's values there as they are projected; v_mode 2
// caches (1 - lambda) v + lambda v_keep with lambda = *v_lambda.
// maps > 1: every head of q and k comes as `maps` heads of hd beside one another, each rotated and normed by
// itself (nh and the key heads of the input count them all, nkv key heads of the pages hold maps * hd channels,
// map m at channel m hd).  q_out row `head` then has its hd numbers at channel (head % maps) hd and zeros
// elsewhere: its score with a page's whole key is the score of its own map.
// v_from_k: there are no values in the input; a kv head's values are its key as projected (with its bias).
// This form takes any size: one wave per (token, head), four waves a block, each with an LDS row of its own; the
// next one takes what comes in pieces of eight channels.
// ---------------------------------------------------------------------------
template <typename T, typename TIN>
__global__ void rope_norm_store_kernel(
    const TIN* __restrict__ qkv, int parts, long part_stride, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, const float* __restrict__ cos_t, const float* __restrict__ sin_t,
    const int* __restrict__ positions, const int* __restrict__ req_of_token,
    const int* __restrict__ block_tables, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, int nh, int nkv_in, int nkv, int hd, int vd, int hdp, int vdp, int rot, int ps,
    int max_pages, int unit, float eps, int num_pairs, int interleaved, float* __restrict__ v_keep, int v_mode,
    const float* __restrict__ v_lambda, long in_ld, const float* __restrict__ bias, int norm_first, int maps,
    int v_from_k) {
  __shared__ float vecs[kPairsPerBlock][kMaxHeadDim];
  const int lane = threadIdx.x & (kWave - 1), wave = threadIdx.x / kWave;
  const int nk_in = nkv_in * maps;
  const int heads = nh + nk_in + nkv_in;
  const int pair = blockIdx.x * kPairsPerBlock + wave;
  if (pair >= num_pairs) return;  // nothing below synchronises across waves
  const int n = pair / heads, head = pair - n * heads;
  float* vec = vecs[wave];
  const bool is_q = head < nh;
  const bool is_k = !is_q && head < nh + nk_in;
  const int width = (is_q || is_k) ? hd : vd;
  const size_t head_at = (is_q || is_k) ? (size_t)head * hd
                         : v_from_k     ? (size_t)(head - nk_in) * hd
                                        : (size_t)(nh + nk_in) * hd + (size_t)(head - nh - nk_in) * vd;
  const TIN* src = qkv + (size_t)n * in_ld + head_at;
  for (int d = lane; d < width; d += kWave) {
    float v = bias ? bias[head_at + d] : 0.f;
    for (int p = 0; p < parts; ++p) v += Elem<TIN>::load(src + (size_t)p * part_stride + d);
    vec[d] = v;
  }
  wave_lds_sync();
  auto norm_head = [&]() {
    float ss = 0.f;
    for (int d = lane; d < hd; d += kWave) ss += vec[d] * vec[d];
    ss = wave_sum(ss);
    const float rstd = 1.f / sqrtf(ss / (float)hd + eps);
    const float* w = is_q ? q_weight : k_weight;
    for (int d = lane; d < hd; d += kWave) vec[d] = vec[d] * rstd * (w ? w[d] : 1.f);   // (a lane rewrites what it read)
    wave_lds_sync();
  };
  if (is_q || is_k) {
    if (unit && norm_first) norm_head();
    const int half = rot / 2;
    float lo[kMaxHeadDim / 2 / kWave], hi[kMaxHeadDim / 2 / kWave];
    int cnt = 0;
    for (int j = lane; j < half; j += kWave, ++cnt) {
      const float c = cos_t[(size_t)n * half + j], s = sin_t[(size_t)n * half + j];
      const float a = vec[interleaved ? 2 * j : j], b = vec[interleaved ? 2 * j + 1 : j + half];
      lo[cnt] = a * c - b * s;
      hi[cnt] = b * c + a * s;
    }
    wave_lds_sync();
    cnt = 0;
    for (int j = lane; j < half; j += kWave, ++cnt) {
      vec[interleaved ? 2 * j : j] = lo[cnt];
      vec[interleaved ? 2 * j + 1 : j + half] = hi[cnt];
    }
    wave_lds_sync();
    if (unit && !norm_first) norm_head();
  }
  if (is_q) {
    T* dst = q_out + ((size_t)n * nh + head) * hdp;
    const int at = (head % maps) * hd;
    for (int d = lane; d < hdp; d += kWave) Elem<T>::store(dst + d, (d >= at && d < at + hd) ? vec[d - at] : 0.f);
    return;
  }
  const int pos = positions[n];
  const int page = block_tables[(size_t)req_of_token[n] * max_pages + pos / ps];
  const int off = pos % ps;
  if (is_k) {
    const int kvh = (head - nh) / maps, at = ((head - nh) % maps) * hd;
    T* base = k_cache + (size_t)page * ((size_t)nkv * hdp * ps) + (size_t)kvh * hdp * ps;
    for (int d = lane; d < hd; d += kWave)
      Elem<T>::store(base + ((size_t)((at + d) >> 3) * ps + off) * 8 + ((at + d) & 7), vec[d]);
  } else {
    const int kvh = head - nh - nk_in;
    T* base = v_cache + (size_t)page * ((size_t)nkv * vdp * ps) + (size_t)kvh * vdp * ps;
    float* keep = v_keep + ((size_t)n * nkv + kvh) * vd;
    const float lambda = v_mode == 2 ? *v_lambda : 0.f;
    for (int d = lane; d < vd; d += kWave) {
      float v = vec[d];
      if (v_mode == 1) keep[d] = v;
      else if (v_mode == 2) v = (1.f - lambda) * v + lambda * keep[d];
      Elem<T>::store(base + ((size_t)(d >> 4) * (ps >> 2) + (off >> 2)) * 64 + (d & 15) * 4 + (off & 3), v);
    }
  }
}

// The same in pieces of eight channels: a lane owns eight neighbouring channels of a head (head sizes that are
// multiples of 8, up to 8 LK channels for queries and keys and 8 LV for values; half-split rotations of multiples of
// 16 dims).  The rotation's partner is in the lane (interleaved pairs) or rot / 16 lanes away.  Blocks of 256 threads:
// the first `key_blocks` take queries, token by token, and behind them the keys, each head with its tokens in order;
// the rest take the values likewise, so that neighbouring lanes hold neighbouring tokens of one head and the cache writes
// fall next to each other; the values of four tokens that fill one quad of a page are exchanged through LDS inside the
// wave and written as the page's own 16-byte pieces of two dims by four keys (bfloat16).
struct RopeNormArgs {
  const float* q_weight;
  const float* k_weight;
  const float* cos_t;
  const float* sin_t;
  const int* positions;
  const int* req_of_token;
  const int* block_tables;
  const float* bias;
  float* v_keep;
  const float* v_lambda;
  long part_stride, in_ld;
  int parts, N, nh, nkv_in, nkv, hd, vd, hdp, vdp, rot, ps, max_pages, unit, interleaved, v_mode, norm_first, maps, v_from_k;
  float eps;
};

template <typename TIN>
__device__ __forceinline__ void load_piece(const TIN* src, int parts, long part_stride, const float* bias, float (&x)[8]) {
  if (bias) {
    const float4 a = *reinterpret_cast<const float4*>(bias), b = *reinterpret_cast<const float4*>(bias + 4);
    x[0] = a.x; x[1] = a.y; x[2] = a.z; x[3] = a.w;
    x[4] = b.x; x[5] = b.y; x[6] = b.z; x[7] = b.w;
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = 0.f;
  }
  for (int p = 0; p < parts; p += 4) {      // four partial sums in flight, added in split order
    float4 a[4], b[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (p + u < parts) {
        a[u] = Load4<TIN>::at(src + (size_t)(p + u) * part_stride);
        b[u] = Load4<TIN>::at(src + (size_t)(p + u) * part_stride + 4);
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (p + u < parts) {
        x[0] += a[u].x; x[1] += a[u].y; x[2] += a[u].z; x[3] += a[u].w;
        x[4] += b[u].x; x[5] += b[u].y; x[6] += b[u].z; x[7] += b[u].w;
      }
    }
  }
}

template <typename T>
__device__ __forceinline__ void store_piece(T* p, const float (&x)[8]) {
  if constexpr (sizeof(T) == 2) {
    *reinterpret_cast<uint4*>(p) = make_uint4(pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3]), pack_bf16x2(x[4], x[5]),
                                              pack_bf16x2(x[6], x[7]));
  } else {
    *reinterpret_cast<float4*>(p) = make_float4(x[0], x[1], x[2], x[3]);
    *reinterpret_cast<float4*>(p + 4) = make_float4(x[4], x[5], x[6], x[7]);
  }
}

template <typename T, typename TIN, int LK, int LV>
__global__ __launch_bounds__(256) void rope_norm_store_vec_kernel(const TIN* __restrict__ in, T* __restrict__ q_out,
                                                                  T* __restrict__ k_cache, T* __restrict__ v_cache,
                                                                  RopeNormArgs A, int key_blocks) {
  __shared__ uint4 s_quad[sizeof(T) == 2 ? 256 : 1];
  const int nk_in = A.nkv_in * A.maps;
  if ((int)blockIdx.x < key_blocks) {
    const unsigned slot = (blockIdx.x * 256u + threadIdx.x) / LK;
    const unsigned q_pairs = (unsigned)A.N * (unsigned)A.nh;
    if (slot >= q_pairs + (unsigned)A.N * (unsigned)nk_in) return;     // (whole groups of LK lanes leave together)
    const int sub = threadIdx.x % LK, d0 = sub * 8;
    int n, head;
    if (slot < q_pairs) {
      n = (int)(slot / (unsigned)A.nh);
      head = (int)(slot - (unsigned)n * (unsigned)A.nh);
    } else {
      const unsigned behind = slot - q_pairs, k = behind / (unsigned)A.N;
      n = (int)(behind - k * (unsigned)A.N);
      head = A.nh + (int)k;
    }
    const bool is_q = head < A.nh, mine = d0 < A.hd;      // (lanes behind the head's end bring zeros)
    const size_t at = (size_t)head * A.hd + d0;
    float x[8];
    if (mine) {
      load_piece<TIN>(in + (size_t)n * A.in_ld + at, A.parts, A.part_stride, A.bias ? A.bias + at : nullptr, x);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = 0.f;
    }
    auto norm_head = [&]() {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += x[e] * x[e];
#pragma unroll
      for (int m = LK / 2; m >= 1; m >>= 1) ss += __shfl_xor(ss, m, kWave);
      const float rstd = 1.f / sqrtf(ss / (float)A.hd + A.eps);
      const float* w = is_q ? A.q_weight : A.k_weight;
      if (w && mine) {
        const float4 w0 = *reinterpret_cast<const float4*>(w + d0), w1 = *reinterpret_cast<const float4*>(w + d0 + 4);
        const float wv[8] = {w0.x, w0.y, w0.z, w0.w, w1.x, w1.y, w1.z, w1.w};
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = x[e] * rstd * wv[e];
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] *= rstd;
      }
    };
    if (A.unit && A.norm_first) norm_head();
    const int half = A.rot / 2;
    if (A.interleaved) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = d0 / 2 + e;
        if (j < half) {
          const float c = A.cos_t[(size_t)n * half + j], s = A.sin_t[(size_t)n * half + j];
          const float a = x[2 * e], b = x[2 * e + 1];
          x[2 * e] = a * c - b * s;
          x[2 * e + 1] = b * c + a * s;
        }
      }
    } else if (half > 0) {
      // (half is a multiple of 8: a lane's piece lies wholly in the first half, the second, or behind)
      const bool first = d0 < half, turns = d0 < A.rot;
      const int partner = (threadIdx.x & 63) + (first ? half / 8 : turns ? -(half / 8) : 0);
      float c[8], s[8];
      if (turns) {
        const size_t j = (size_t)n * half + (first ? d0 : d0 - half);
        const float4 c0 = *reinterpret_cast<const float4*>(A.cos_t + j), c1 = *reinterpret_cast<const float4*>(A.cos_t + j + 4);
        const float4 s0 = *reinterpret_cast<const float4*>(A.sin_t + j), s1 = *reinterpret_cast<const float4*>(A.sin_t + j + 4);
        c[0] = c0.x; c[1] = c0.y; c[2] = c0.z; c[3] = c0.w; c[4] = c1.x; c[5] = c1.y; c[6] = c1.z; c[7] = c1.w;
        s[0] = s0.x; s[1] = s0.y; s[2] = s0.z; s[3] = s0.w; s[4] = s1.x; s[5] = s1.y; s[6] = s1.z; s[7] = s1.w;
      }
      const float sign = first ? -1.f : 1.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float other = __shfl(x[e], partner, kWave);
        if (turns) x[e] = x[e] * c[e] + sign * other * s[e];
      }
    }
    if (A.unit && !A.norm_first) norm_head();
    if (!mine) return;
    if (is_q) {
      T* dst = q_out + ((size_t)n * A.nh + head) * A.hdp + d0;
      const int map = head % A.maps;
      const float zero[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      for (int m = 0; m < A.maps; ++m) {
        if (m == map) store_piece<T>(dst + m * A.hd, x);
        else store_piece<T>(dst + m * A.hd, zero);
      }
      return;
    }
    const int pos = A.positions[n];
    const int page = A.block_tables[(size_t)A.req_of_token[n] * A.max_pages + pos / A.ps], off = pos % A.ps;
    const int kvh = (head - A.nh) / A.maps, piece = ((head - A.nh) % A.maps) * (A.hd / 8) + sub;
    store_piece<T>(k_cache + (size_t)page * ((size_t)A.nkv * A.hdp * A.ps) + (size_t)kvh * A.hdp * A.ps +
                       ((size_t)piece * A.ps + off) * 8, x);
    return;
  }
  const unsigned slot = ((blockIdx.x - (unsigned)key_blocks) * 256u + threadIdx.x) / LV;
  if (slot >= (unsigned)A.N * (unsigned)A.nkv_in) return;
  const int sub = threadIdx.x % LV, d0 = sub * 8;
  const int kvh = (int)(slot / (unsigned)A.N), n = (int)(slot - (unsigned)kvh * (unsigned)A.N);
  const bool mine = d0 < A.vd;
  const size_t at = A.v_from_k ? (size_t)(A.nh + kvh) * A.hd + d0 : (size_t)(A.nh + nk_in) * A.hd + (size_t)kvh * A.vd + d0;
  float x[8];
  if (mine) {
    load_piece<TIN>(in + (size_t)n * A.in_ld + at, A.parts, A.part_stride, A.bias ? A.bias + at : nullptr, x);
    if (A.v_mode) {
      float* keep = A.v_keep + ((size_t)n * A.nkv + kvh) * A.vd + d0;
      const float lambda = A.v_mode == 2 ? *A.v_lambda : 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        if (A.v_mode == 1) keep[e] = x[e];
        else x[e] = (1.f - lambda) * x[e] + lambda * keep[e];
      }
    }
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) x[e] = 0.f;
  }
  const int pos = A.positions[n], req = A.req_of_token[n];
  const int page = A.block_tables[(size_t)req * A.max_pages + pos / A.ps], off = pos % A.ps;
  T* base = v_cache + (size_t)page * ((size_t)A.nkv * A.vdp * A.ps) + (size_t)kvh * A.vdp * A.ps;
  if constexpr (sizeof(T) == 2 && LV <= 16) {
    // four tokens in a row (a "quad" of this wave) of one request and head that fill one quad of keys in a page?
    constexpr int QL = 4 * LV;
    const int lane = threadIdx.x & 63, t = (lane / LV) & 3;
    const int lead = lane / QL * QL + sub;             // the lane with these dims in the quad's first token
    const bool fits = n == __shfl(n, lead, kWave) + t && pos == __shfl(pos, lead, kWave) + t &&
                      req == __shfl(req, lead, kWave) && kvh == __shfl(kvh, lead, kWave) && ((pos - t) & 3) == 0;
    const unsigned long long all = QL == 64 ? ~0ull : ((1ull << (QL & 63)) - 1) << (lane / QL * QL);
    if ((__builtin_amdgcn_ballot_w64(fits) & all) == all) {
      s_quad[threadIdx.x] = make_uint4(pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3]), pack_bf16x2(x[4], x[5]),
                                       pack_bf16x2(x[6], x[7]));
      wave_lds_sync();
      const unsigned* words = reinterpret_cast<const unsigned*>(s_quad);
      const int quad0 = (int)threadIdx.x / QL * QL + sub;
      unsigned r[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) r[k] = words[(quad0 + k * LV) * 4 + t];      // token k: dims d, d + 1
      const int d = d0 + 2 * t;
      uint4 piece;      // [dim d: keys 0..3][dim d + 1: keys 0..3]
      piece.x = (r[0] & 0xffffu) | (r[1] << 16);
      piece.y = (r[2] & 0xffffu) | (r[3] << 16);
      piece.z = (r[0] >> 16) | (r[1] & 0xffff0000u);
      piece.w = (r[2] >> 16) | (r[3] & 0xffff0000u);
      if (mine) *reinterpret_cast<uint4*>(base + ((size_t)(d >> 4) * (A.ps >> 2) + (off >> 2)) * 64 + (d & 15) * 4) = piece;
      return;
    }
  }
  if (!mine) return;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const int d = d0 + e;
    Elem<T>::store(base + ((size_t)(d >> 4) * (A.ps >> 2) + (off >> 2)) * 64 + (d & 15) * 4 + (off & 3), x[e]);
  }
}

static bool rope_norm_vec_fits(const RopeNormArgs& A, const void* in, const void* q_out, const void* k_cache, const void* v_cache,
                               int in_bytes) {
  auto aligned = [](const void* p) { return (uintptr_t)p % 16 == 0; };
  return A.hd % 8 == 0 && A.hd <= 256 && A.hdp == A.maps * A.hd && (A.nkv_in == 0 || (A.vd % 8 == 0 && A.vd <= 256)) &&
         (A.interleaved || (A.rot / 2) % 8 == 0) && A.in_ld * in_bytes % 16 == 0 && A.part_stride * in_bytes % 16 == 0 &&
         A.ps % 8 == 0 && aligned(in) && aligned(q_out) && aligned(k_cache) && aligned(v_cache) && aligned(A.cos_t) &&
         aligned(A.sin_t) && aligned(A.bias) && aligned(A.q_weight) && aligned(A.k_weight);
}

template <typename T, typename TIN, int LK>
static void launch_rope_norm_vec(const void* in, void* q_out, void* k_cache, void* v_cache, const RopeNormArgs& A, hipStream_t stream) {
  const long key_pairs = (long)A.N * (A.nh + (long)A.nkv_in * A.maps), value_pairs = (long)A.N * A.nkv_in;
  const int lv = A.vd <= 64 ? 8 : A.vd <= 128 ? 16 : 32;
  const long key_blocks = (key_pairs * LK + 255) / 256, value_blocks = (value_pairs * lv + 255) / 256;
#define TK_RV(LV_)                                                                                                   \
  rope_norm_store_vec_kernel<T, TIN, LK, LV_><<<(unsigned)(key_blocks + value_blocks), 256, 0, stream>>>(            \
      (const TIN*)in, (T*)q_out, (T*)k_cache, (T*)v_cache, A, (int)key_blocks)
  if (lv == 8) TK_RV(8);
  else if (lv == 16) TK_RV(16);
  else TK_RV(32);
#undef TK_RV
}

// in_f32: qkv is float32 (possibly `parts` partial sums, part_stride elements apart)
TK_API int tk_rope_norm_store(int dtype, const void* qkv, int in_f32, int parts, long part_stride,
                              const float* q_weight, const float* k_weight, const float* cos_t,
                              const float* sin_t, const int* positions, const int* req_of_token,
                              const int* block_tables, void* q_out, void* k_cache, void* v_cache,
                              int N, int nh, int nkv_in, int nkv, int hd, int vd, int hdp, int vdp, int rot,
                              int ps, int max_pages, int unit, float eps, int interleaved, float* v_keep,
                              int v_mode, const float* v_lambda, long in_ld, const float* bias, int norm_first,
                              int maps, int v_from_k, hipStream_t stream) {
  if (N <= 0) return 0;
  if (maps < 1 || nh % maps != 0 || (v_from_k && (maps != 1 || vd != hd))) return -1;
  if (hdp > kMaxHeadDim || vdp > kMaxHeadDim || hd < 1 || vd < 1 || (long)hdp < (long)maps * hd || vdp < vd || hdp % 8 != 0 ||
      vdp % 16 != 0 || ps % 4 != 0 || rot > hd || rot % 2 != 0)
    return -1;
  if (v_mode < 0 || v_mode > 2 || (v_mode != 0 && v_keep == nullptr) || (v_mode == 2 && v_lambda == nullptr)) return -1;
  if (nkv_in != 0 && nkv_in != nkv) return -1;
  if (parts < 1 || (parts > 1 && !in_f32 && dtype != 0)) return -1;
  if (in_ld < ((long)nh + (long)nkv_in * maps) * hd + (v_from_k ? 0L : (long)nkv_in * vd)) return -1;
  const long pairs = (long)N * (nh + (long)nkv_in * (maps + 1));
  if (pairs > 0x7fffffffL) return -1;
  const RopeNormArgs args{q_weight, k_weight, cos_t, sin_t, positions, req_of_token, block_tables, bias, v_keep, v_lambda,
                          part_stride, in_ld, parts, N, nh, nkv_in, nkv, hd, vd, hdp, vdp, rot, ps, max_pages, unit,
                          interleaved, v_mode, norm_first, maps, v_from_k, eps};
  if (rope_norm_vec_fits(args, qkv, q_out, k_cache, v_cache, dtype == 0 || in_f32 ? 4 : 2) && pairs <= (1L << 26)) {
#define TK_RK(T_, TIN_)                                                                                        \
  {                                                                                                            \
    if (hd <= 64) launch_rope_norm_vec<T_, TIN_, 8>(qkv, q_out, k_cache, v_cache, args, stream);               \
    else if (hd <= 128) launch_rope_norm_vec<T_, TIN_, 16>(qkv, q_out, k_cache, v_cache, args, stream);        \
    else launch_rope_norm_vec<T_, TIN_, 32>(qkv, q_out, k_cache, v_cache, args, stream);                       \
  }
    if (dtype == 0) TK_RK(float, float)
    else if (in_f32) TK_RK(bf16_t, float)
    else TK_RK(bf16_t, bf16_t)
#undef TK_RK
    return launch_status();
  }
  const unsigned grid = (unsigned)((pairs + kPairsPerBlock - 1) / kPairsPerBlock);
#define TK_RN(T_, TIN_)                                                                          \
  rope_norm_store_kernel<T_, TIN_><<<grid, kWave * kPairsPerBlock, 0, stream>>>(                 \
      (const TIN_*)qkv, parts, part_stride, q_weight, k_weight, cos_t, sin_t, positions,         \
      req_of_token, block_tables, (T_*)q_out, (T_*)k_cache, (T_*)v_cache, nh, nkv_in, nkv, hd,   \
      vd, hdp, vdp, rot, ps, max_pages, unit, eps, (int)pairs, interleaved, v_keep, v_mode, v_lambda, in_ld, bias, norm_first, maps, v_from_k)
  if (dtype == 0) TK_RN(float, float);
  else if (in_f32) TK_RN(bf16_t, float);
  else TK_RN(bf16_t, bf16_t);
#undef TK_RN
  return launch_status();
}

// ---------------------------------------------------------------------------
// logits in place: x <- x * scale, then (cap > 0) x <- cap * tanh(x / cap)
// ---------------------------------------------------------------------------
__global__ void scale_softcap_kernel(float* __restrict__ x, size_t total, float scale, float cap) {
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  float v = x[idx] * scale;
  if (cap > 0.f) v = cap * tanhf(v / cap);
  x[idx] = v;
}

TK_API int tk_scale_softcap(float* x, long total, float scale, float cap, hipStream_t stream) {
  if (total <= 0) return 0;
  scale_softcap_kernel<<<(unsigned)((total + 255) / 256), 256, 0, stream>>>(x, (size_t)total, scale, cap);
  return launch_status();
}

// the same entry points in slot form (slots.h), for launch lists
TK_SLOTS(tk_add_rmsnorm)
TK_SLOTS(tk_add_norm2)
TK_SLOTS(tk_add_normed)
TK_SLOTS(tk_sigmoid_gate)
TK_SLOTS(tk_rope_tables)
TK_SLOTS(tk_qknorm_rope_store)
TK_SLOTS(tk_silu_mul)
TK_SLOTS(tk_silu_mul_parts)
TK_SLOTS(tk_add_bias)
TK_SLOTS(tk_squared_relu)
TK_SLOTS(tk_map_difference)
TK_SLOTS(tk_scaled_sum)
TK_SLOTS(tk_rope_norm_store)
TK_SLOTS(tk_scale_softcap)
