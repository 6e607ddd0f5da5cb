// Kernels of the gated delta rule with a decay per key channel (gfx950).
//
// The mixer's products leave, per token, [q | k | v | b] (proj) and [z | gate] (up).
//
// delta_inputs: q, k and v pass a short causal convolution per channel and SiLU (the last tap meets the token
//   itself; the inputs before a step's first token come from the request's state, zeros at a sequence's start); q
//   and k become unit vectors per head, x / sqrt(sum(x^2) + 1e-6), q times q_scale; the decay of a key channel is
//   exp(-exp(A_log) softplus(z + dt_bias)); beta = sigmoid(b).  All of it lands in one float32 row per token,
//   [q: kv dim | k: kv dim | v: heads vdim | decay: heads dim | beta: heads], rounded up to a multiple of four.
// delta_scan: per (request, head), over the step's tokens in order, with the state S [dim, vdim] in float32
//   registers (q and k of kv head head / (heads / kv)):
//     S <- diag(decay) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.
//
// Convolution, norms, decays with their exponentials, beta, the recurrence and its state are float32 whatever
// the storage type.
#include "common.h"
#include "short_conv.h"
#include "slots.h"

using namespace tk;

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));   // (arrays of HIP's float4 struct may end up in scratch)

constexpr int kSegment = 16;      // tokens of a request that a wave of delta_inputs walks
constexpr int kTogether = 4;      // of which a wave asks for this many together
constexpr float kUnitEps = 1e-6f;

struct DeltaShape {
  int heads, kv, dim, vdim, taps;
  __host__ __device__ int conv_channels() const { return 2 * kv * dim + heads * vdim; }
  __host__ __device__ int row() const { return (2 * kv * dim + heads * vdim + heads * dim + heads + 3) / 4 * 4; }   // (whole 16-byte pieces)
};

// A wave a unit (a q or k head, or a run of 64 * CPL channels of v or of the decays) and a segment of a request's
// tokens: a lane walks CPL channels with the taps' inputs in registers.  grid (units / 4, requests, segments).
// update: a request's tokens are this one segment, whose wave also writes the convolution's new state.
// WIDE: a lane's channels are neighbours and read and written as one piece (every width a multiple of CPL); else lane,
// lane + 64, ...
template <typename T, int N> struct Piece { using type = void; };
template <> struct Piece<bf16_t, 1> { using type = uint16_t; };
template <> struct Piece<bf16_t, 2> { using type = uint32_t; };
template <> struct Piece<bf16_t, 4> { using type = uint2; };
template <> struct Piece<float, 1> { using type = float; };
template <> struct Piece<float, 2> { using type = float2; };
template <> struct Piece<float, 4> { using type = float4; };

// N neighbouring elements from idx on of rows in T, float32 or partial sums
template <typename T, int N>
__device__ __forceinline__ void load_piece(const RowsIn& in, size_t idx, float (&v)[N]) {
  if (!in.f32) {
    union { typename Piece<bf16_t, N>::type u; bf16_t e[N]; } p;
    p.u = *reinterpret_cast<const typename Piece<bf16_t, N>::type*>(reinterpret_cast<const bf16_t*>(in.p) + idx);
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = bf16_to_float(p.e[i]);
    return;
  }
  const float* f = reinterpret_cast<const float*>(in.p) + idx;
#pragma unroll
  for (int i = 0; i < N; ++i) v[i] = 0.f;
  for (int k = 0; k < in.parts; ++k) {
    union { typename Piece<float, N>::type u; float e[N]; } p;
    p.u = *reinterpret_cast<const typename Piece<float, N>::type*>(f + (size_t)k * in.stride);
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] += p.e[i];
  }
}
template <int N>
__device__ __forceinline__ void store_piece(float* dst, const float (&v)[N]) {
  union { typename Piece<float, N>::type u; float e[N]; } p;
#pragma unroll
  for (int i = 0; i < N; ++i) p.e[i] = v[i];
  *reinterpret_cast<typename Piece<float, N>::type*>(dst) = p.u;
}

// A lane's CPL channels of a unit's `count`, from `at` on (channels that do not exist: zeros, not stored).
template <typename T, int CPL, bool WIDE>
__device__ __forceinline__ void load_channels(const RowsIn& in, size_t at, int lane, int count, float (&v)[CPL]) {
  if constexpr (WIDE) {
#pragma unroll
    for (int i = 0; i < CPL; ++i) v[i] = 0.f;
    if (lane * CPL < count) load_piece<T, CPL>(in, at + lane * CPL, v);
  } else {
#pragma unroll
    for (int i = 0; i < CPL; ++i) v[i] = i * kWave + lane < count ? load_in<T>(in, at + i * kWave + lane) : 0.f;
  }
}
template <int CPL, bool WIDE>
__device__ __forceinline__ void store_channels(float* dst, int lane, int count, const float (&v)[CPL]) {
  if constexpr (WIDE) {
    if (lane * CPL < count) store_piece<CPL>(dst + lane * CPL, v);
  } else {
#pragma unroll
    for (int i = 0; i < CPL; ++i)
      if (i * kWave + lane < count) dst[i * kWave + lane] = v[i];
  }
}

// TAPS: at least the convolution's taps.  Four tokens' inputs are asked for together.
template <typename T, int CPL, int TAPS, bool WIDE>
__global__ __launch_bounds__(256) void delta_inputs_kernel(
    RowsIn proj, long ld, RowsIn up, long uld, const float* __restrict__ conv, float* __restrict__ state,
    const float* __restrict__ a_log, const float* __restrict__ dt_bias, const int* __restrict__ q_start,
    const int* __restrict__ state_slots, float* __restrict__ out, DeltaShape sh, float q_scale, int update) {
  const int lane = threadIdx.x & (kWave - 1);
  int unit = blockIdx.x * (blockDim.x / kWave) + threadIdx.x / kWave;
  const int req = blockIdx.y;
  const int first = q_start[req], end = q_start[req + 1];
  const int t_lo = first + blockIdx.z * kSegment, t_hi = min(end, t_lo + kSegment);
  if (t_lo >= end) return;                 // (nothing below synchronises across waves)
  constexpr int RUN = kWave * CPL;
  const int kdim = sh.kv * sh.dim, vall = sh.heads * sh.vdim, gall = sh.heads * sh.dim;
  const int vunits = (vall + RUN - 1) / RUN, gunits = (gall + RUN - 1) / RUN;
  const int C = sh.conv_channels(), row = sh.row(), taps = sh.taps;
  if (unit >= 2 * sh.kv + vunits) {
    unit -= 2 * sh.kv + vunits;
    if (unit >= gunits) return;
    // decays, and (its first unit) the heads' step sizes
    float* dst = out + C;
    const int from = unit * RUN, count = min(RUN, gall - from);
    float rate[CPL], bias[CPL];
#pragma unroll
    for (int i = 0; i < CPL; ++i) {
      const int c = WIDE ? lane * CPL + i : i * kWave + lane;
      rate[i] = c < count ? expf(a_log[(from + c) / sh.dim]) : 0.f;
      bias[i] = c < count ? dt_bias[from + c] : 0.f;
    }
    for (int t0 = t_lo; t0 < t_hi; t0 += kTogether) {
      float z[kTogether][CPL];
#pragma unroll
      for (int u = 0; u < kTogether; ++u)      // (a row behind the last token's: the last token's again)
        load_channels<T, CPL, WIDE>(up, (size_t)min(t0 + u, t_hi - 1) * uld + from, lane, count, z[u]);
#pragma unroll
      for (int u = 0; u < kTogether; ++u) {
        if (t0 + u >= t_hi) break;
#pragma unroll
        for (int i = 0; i < CPL; ++i) z[u][i] = __expf(-rate[i] * softplus(z[u][i] + bias[i]));
        store_channels<CPL, WIDE>(dst + (size_t)(t0 + u) * row + from, lane, count, z[u]);
      }
    }
    if (unit == 0) {
      for (int i = lane; i < (t_hi - t_lo) * sh.heads; i += kWave) {
        const int t = t_lo + i / sh.heads, head = i % sh.heads;
        out[(size_t)t * row + C + gall + head] = sigmoid(load_in<T>(proj, (size_t)t * ld + C + head));
      }
    }
    return;
  }
  const bool qk = unit < 2 * sh.kv;
  const int col0 = qk ? unit * sh.dim : 2 * kdim + (unit - 2 * sh.kv) * RUN;     // (q's heads, then k's)
  const int count = qk ? sh.dim : min(RUN, vall - (unit - 2 * sh.kv) * RUN);
  const float scale = unit < sh.kv ? q_scale : 1.f;
  float* st = taps > 1 ? state + (size_t)state_slots[req] * (taps - 1) * C + col0 : nullptr;
  // taps sit at the END of arrays of TAPS: index TAPS - 1 is the token itself; win holds the inputs of the TAPS - 1
  // positions before a group of kTogether tokens, and then theirs
  float wv[TAPS][CPL], win[TAPS - 1 + kTogether][CPL];
#pragma unroll
  for (int k = 0; k < TAPS; ++k) {
    const int j = k - (TAPS - taps);
#pragma unroll
    for (int i = 0; i < CPL; ++i) {
      const int c = WIDE ? lane * CPL + i : i * kWave + lane;
      wv[k][i] = (j >= 0 && c < count) ? conv[(size_t)(col0 + c) * taps + j] : 0.f;
    }
  }
#pragma unroll
  for (int d = 1; d < TAPS; ++d) {
    const int local = t_lo - first - d;       // the input d positions before the segment's first token
    if (d < taps && local >= 0) {
      load_channels<T, CPL, WIDE>(proj, (size_t)(t_lo - d) * ld + col0, lane, count, win[TAPS - 1 - d]);
    } else {
#pragma unroll
      for (int i = 0; i < CPL; ++i) {
        const int c = WIDE ? lane * CPL + i : i * kWave + lane;
        win[TAPS - 1 - d][i] = d < taps && c < count ? st[(size_t)(taps - 1 + local) * C + c] : 0.f;
      }
    }
  }
  for (int t0 = t_lo; t0 < t_hi; t0 += kTogether) {
    const int many = min(kTogether, t_hi - t0);
#pragma unroll
    for (int u = 0; u < kTogether; ++u)      // (a row behind the last token's: the last token's again, not used)
      load_channels<T, CPL, WIDE>(proj, (size_t)min(t0 + u, t_hi - 1) * ld + col0, lane, count, win[TAPS - 1 + u]);
    float y[kTogether][CPL], ss[kTogether];
#pragma unroll
    for (int u = 0; u < kTogether; ++u) {
      ss[u] = 0.f;
#pragma unroll
      for (int i = 0; i < CPL; ++i) {
        float acc = 0.f;
#pragma unroll
        for (int k = 0; k < TAPS; ++k) acc = fmaf(wv[k][i], win[u + k][i], acc);
        y[u][i] = silu(acc);        // (channels behind the unit's: zero)
        ss[u] = fmaf(y[u][i], y[u][i], ss[u]);
      }
    }
    if (qk) {
#pragma unroll
      for (int u = 0; u < kTogether; ++u) {
        const float r = scale / sqrtf(wave_sum(ss[u]) + kUnitEps);
#pragma unroll
        for (int i = 0; i < CPL; ++i) y[u][i] *= r;
      }
    }
#pragma unroll
    for (int u = 0; u < kTogether; ++u)
      if (u < many) store_channels<CPL, WIDE>(out + (size_t)(t0 + u) * row + col0, lane, count, y[u]);
    // the window moves on by the tokens that were there
#pragma unroll
    for (int u = 1; u <= kTogether; ++u) {
      if (u == many) {
#pragma unroll
        for (int k = 0; k < TAPS - 1; ++k)
#pragma unroll
          for (int i = 0; i < CPL; ++i) win[k][i] = win[k + u][i];
      }
    }
  }
  if (update) {      // (the window now ends at the request's last token)
#pragma unroll
    for (int k = 0; k < TAPS - 1; ++k) {
      const int j = k - (TAPS - taps);
      if (j >= 0) store_channels<CPL, WIDE>(st + (size_t)j * C, lane, count, win[k]);
    }
  }
}

// Sum over each run of 16 neighbouring lanes, in every lane of the run: quads by permutation, then the mirrored
// half of eight and of sixteen (after each step all lanes of the mirrored group hold the same number).
template <int CTRL>
__device__ __forceinline__ float lane_move(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float sum16(float v) {
  v += lane_move<0xB1>(v);       // quad_perm [1, 0, 3, 2]
  v += lane_move<0x4E>(v);       // quad_perm [2, 3, 0, 1]
  v += lane_move<0x141>(v);      // row_half_mirror
  v += lane_move<0x140>(v);      // row_mirror
  return v;
}

constexpr int kLanes = 16;        // lanes that share a value column
constexpr int kColumns = 16;      // value columns of a block of four waves
constexpr int kScanThreads = 256;

// One round's operands, tokens t0 .. t0 + tb, on their way from memory: piece e of the round is
// [k | q | decay] as [TB][DP / 4] each, then v as [TB][4].  *_at: where they lie in a token's row; columns: the value
// columns that exist from the block's first one on.
template <int PER, int TB, int DP, bool WIDE>
__device__ __forceinline__ void fetch_round(const float* __restrict__ in, int row, int k_at, int q_at, int g_at,
                                            int v_at, int b_at, int dim, int columns, int t0, int tb,
                                            f32x4 (&held)[PER], float& beta) {
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int e = i * kScanThreads + threadIdx.x;
    int t, c, most, from;
    if (e < 3 * TB * DP / 4) {
      const int set = e / (TB * DP / 4), in_set = e - set * (TB * DP / 4);
      t = in_set / (DP / 4);
      c = (in_set - t * (DP / 4)) * 4;
      most = dim;
      from = set == 0 ? k_at : set == 1 ? q_at : g_at;
    } else {
      t = (e - 3 * TB * DP / 4) / (kColumns / 4);
      c = ((e - 3 * TB * DP / 4) - t * (kColumns / 4)) * 4;
      most = columns;
      from = v_at;
    }
    if (t >= tb) most = 0;
    const float* p = in + (size_t)(t0 + t) * row + from + c;
    held[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (WIDE) {
      if (c < most) held[i] = *reinterpret_cast<const f32x4*>(p);
    } else {
      if (c < most) held[i].x = p[0];
      if (c + 1 < most) held[i].y = p[1];
      if (c + 2 < most) held[i].z = p[2];
      if (c + 3 < most) held[i].w = p[3];
    }
  }
  beta = (int)threadIdx.x < tb ? in[(size_t)(t0 + threadIdx.x) * row + b_at] : 0.f;
}

// What a lane reads of a token of the round.
template <int PIECES>
struct DeltaToken {
  f32x4 k[PIECES], q[PIECES], g[PIECES];
  float beta, v;
};

template <int PIECES, int TB>
__device__ __forceinline__ void read_token(const float* lds, const float* vv, const float* bb, int t, int ks, int jl,
                                           DeltaToken<PIECES>& x) {
  constexpr int DP = kLanes * 4 * PIECES, SET = TB * DP;
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int piece = t * DP + i * (kLanes * 4) + ks * 4;
    x.k[i] = *reinterpret_cast<const f32x4*>(lds + piece);
    x.g[i] = *reinterpret_cast<const f32x4*>(lds + 2 * SET + piece);
    x.q[i] = *reinterpret_cast<const f32x4*>(lds + SET + piece);
  }
  x.beta = bb[t];
  x.v = vv[t * kColumns + jl];
}

// The lane's rows of the state move on by a token; its output (the same number in all lanes of the column).
template <int PIECES>
__device__ __forceinline__ float delta_token(const DeltaToken<PIECES>& x, f32x4 (&s)[PIECES]) {
  // Measured on 2,048 tokens of 32 heads of 128 x 128: operands read where they are used 450 us, in a loop that asks for
  // them a token ahead 525 (copies and addresses), unrolled with the reads ahead 370; the rest is the chain itself.
  float d0 = 0.f, d1 = 0.f, o0 = 0.f, o1 = 0.f;
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    s[i] *= x.g[i];
    d0 = fmaf(s[i].x, x.k[i].x, d0);
    d1 = fmaf(s[i].y, x.k[i].y, d1);
    d0 = fmaf(s[i].z, x.k[i].z, d0);
    d1 = fmaf(s[i].w, x.k[i].w, d1);
  }
  const float u = x.beta * (x.v - sum16(d0 + d1));
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    s[i] = f32x4{fmaf(x.k[i].x, u, s[i].x), fmaf(x.k[i].y, u, s[i].y), fmaf(x.k[i].z, u, s[i].z), fmaf(x.k[i].w, u, s[i].w)};
    o0 = fmaf(s[i].x, x.q[i].x, o0);
    o1 = fmaf(s[i].y, x.q[i].y, o1);
    o0 = fmaf(s[i].z, x.q[i].z, o0);
    o1 = fmaf(s[i].w, x.q[i].w, o1);
  }
  return sum16(o0 + o1);
}

// A block a (request, head, 16 value columns).  The 16 neighbouring lanes that share a column hold its rows of the
// state in registers, PIECES pieces of four rows a lane (lane l: rows 64 i + 4 l .. + 4), so that both dot
// products of a token are sums of 4 PIECES multiply-adds and four lane moves, with no LDS and no barrier in
// between.  The tokens' k, q and decays are staged in LDS, TB at a time, the next round's on their way
// to registers meanwhile; the columns of a head never meet, so a head's blocks run side by side.
// The state lies as [head][column][dim rounded up to 4].
// WIDE: dim and vdim are multiples of four, so that rows are read in 16-byte pieces.
template <int PIECES, int TB, bool WIDE>
__global__ __launch_bounds__(kScanThreads, 1) void delta_scan_kernel(
    const float* __restrict__ in, float* __restrict__ state, const int* __restrict__ q_start,
    const int* __restrict__ state_slots, float* __restrict__ y, DeltaShape sh) {
  constexpr int DP = kLanes * 4 * PIECES;      // rows with the padding (zeros behind dim)
  constexpr int SET = TB * DP;
  constexpr int ALL = (3 * SET + TB * kColumns) / 4;      // pieces of four numbers that a round stages
  constexpr int PER = (ALL + kScanThreads - 1) / kScanThreads;
  __shared__ __attribute__((aligned(16))) float lds[3 * SET + TB * kColumns + TB];
  float* vv = lds + 3 * SET;
  float* bb = vv + TB * kColumns;
  const int req = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
  const int first = q_start[req], end = q_start[req + 1];
  const int ks = tid & (kLanes - 1), jl = tid / kLanes;
  const int col0 = blockIdx.z * kColumns, j = col0 + jl;
  const int dim = sh.dim, vdim = sh.vdim, row = sh.row();
  const int rows4 = (dim + 3) & ~3;
  const bool owns = j < vdim;
  const int kvh = head / (sh.heads / sh.kv);
  const int kdim = sh.kv * dim, gall = sh.heads * dim;
  const int behind = 2 * kdim + sh.heads * vdim;      // of q, k and v
  const int q_at = kvh * dim, k_at = kdim + q_at, v_at = 2 * kdim + head * vdim + col0, g_at = behind + head * dim;
  const int b_at = behind + gall + head;
  float* S = state + (((size_t)state_slots[req] * sh.heads + head) * vdim + (owns ? j : 0)) * rows4;
  f32x4 s[PIECES];
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int r = i * (kLanes * 4) + ks * 4;
    s[i] = owns && r < rows4 ? *reinterpret_cast<const f32x4*>(S + r) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  f32x4 held[PER];
  float held_beta = 0.f;
  fetch_round<PER, TB, DP, WIDE>(in, row, k_at, q_at, g_at, v_at, b_at, dim, vdim - col0, first, min(TB, end - first), held, held_beta);
  for (int t0 = first; t0 < end; t0 += TB) {
    const int tb = min(TB, end - t0);
    __syncthreads();     // (the round before has been read)
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int e = i * kScanThreads + tid;
      if (e < ALL) *reinterpret_cast<f32x4*>(lds + 4 * e) = held[i];
    }
    if (tid < TB) bb[tid] = held_beta;
    __syncthreads();
    if (t0 + TB < end) fetch_round<PER, TB, DP, WIDE>(in, row, k_at, q_at, g_at, v_at, b_at, dim, vdim - col0, t0 + TB,
                                                      min(TB, end - t0 - TB), held, held_beta);
    float kept = 0.f;
    DeltaToken<PIECES> x[2];
    read_token<PIECES, TB>(lds, vv, bb, 0, ks, jl, x[0]);
    if (tb == TB) {
      // a whole round, unrolled: a token's operands are read while the token before it is computed (the barrier lets
      // arithmetic pass, LDS reads not: left alone the compiler puts the reads right ahead of their use)
#pragma unroll
      for (int t = 0; t < TB; ++t) {
        if (t + 1 < TB) read_token<PIECES, TB>(lds, vv, bb, t + 1, ks, jl, x[(t + 1) & 1]);
        __builtin_amdgcn_sched_barrier(0x7);
        const float o = delta_token<PIECES>(x[t & 1], s);
        if (ks == t) kept = o;      // (lane t of a column keeps token t's output: one store a round)
      }
    } else {
      for (int t = 0; t < tb; ++t) {
        if (t > 0) read_token<PIECES, TB>(lds, vv, bb, t, ks, jl, x[0]);
        const float o = delta_token<PIECES>(x[0], s);
        if (ks == t) kept = o;
      }
    }
    static_assert(TB <= kLanes, "a lane of a column keeps one token's output");
    if (owns && ks < tb) y[(size_t)(t0 + ks) * sh.heads * vdim + (size_t)head * vdim + j] = kept;
  }
  if (owns) {
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
      const int r = i * (kLanes * 4) + ks * 4;
      if (r < rows4) *reinterpret_cast<f32x4*>(S + r) = s[i];
    }
  }
}

// out[n][c] = the sum of a split product's partial sums at column col0 + c, rounded to T
template <typename T>
__global__ __launch_bounds__(256) void sum_columns_kernel(RowsIn in, long ld, int col0, T* __restrict__ out, int width, long total) {
  const long idx = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= total) return;
  const long n = idx / width;
  Elem<T>::store(out + idx, load_in<T>(in, (size_t)n * ld + col0 + (idx - n * width)));
}

template <typename T>
int launch_inputs(RowsIn proj, long ld, RowsIn up, long uld, const float* conv, float* state, const float* a_log,
                  const float* dt_bias, const int* q_start, const int* slots, float* out, int R, DeltaShape sh,
                  float q_scale, int max_tokens, hipStream_t stream) {
  const int segments = (max_tokens + kSegment - 1) / kSegment;
  const int update = segments == 1 && sh.taps > 1;
  const int cpl = sh.dim <= 64 ? 1 : sh.dim <= 128 ? 2 : sh.dim <= 256 ? 4 : 8;
  const int run = kWave * cpl;
  const long units = 2L * sh.kv + ((long)sh.heads * sh.vdim + run - 1) / run + ((long)sh.heads * sh.dim + run - 1) / run;
  const dim3 grid((unsigned)((units + 3) / 4), R, segments);
  if (grid.y > 65535 || grid.z > 65535) return -1;
  // (every unit then starts on a border of CPL elements in all of its arrays)
  const bool wide = cpl <= 4 && sh.dim % cpl == 0 && sh.heads * sh.vdim % cpl == 0 && ld % cpl == 0 && uld % cpl == 0 &&
                    proj.stride % cpl == 0 && up.stride % cpl == 0 && (uintptr_t)proj.p % 16 == 0 &&
                    (uintptr_t)up.p % 16 == 0 && (uintptr_t)state % 16 == 0 && (uintptr_t)out % 16 == 0;
#define TK_DI_AS(CPL, TAPS, WIDE)                                                                                      \
  delta_inputs_kernel<T, CPL, TAPS, WIDE><<<grid, 256, 0, stream>>>(proj, ld, up, uld, conv, state, a_log, dt_bias, q_start, \
                                                                    slots, out, sh, q_scale, update)
#define TK_DI(CPL, WIDE)                        \
  {                                             \
    if (sh.taps <= 4) TK_DI_AS(CPL, 4, WIDE);   \
    else TK_DI_AS(CPL, kMaxTaps, WIDE);         \
  }
  if (cpl == 1) TK_DI(1, false)
  else if (cpl == 2 && wide) TK_DI(2, true)
  else if (cpl == 2) TK_DI(2, false)
  else if (cpl == 4 && wide) TK_DI(4, true)
  else if (cpl == 4) TK_DI(4, false)
  else TK_DI(8, false)
#undef TK_DI_AS
#undef TK_DI
  if (!update && sh.taps > 1) {
    const int C = sh.conv_channels();
    conv_carry_kernel<T><<<dim3((C + 255) / 256, R), 256, 0, stream>>>(proj, ld, 0, state, q_start, slots, C, sh.taps);
  }
  return launch_status();
}

}  // namespace

// in: float32 [parts, N, ld], parts part_stride elements apart; out [N, width] in dtype: the sums of columns col0 .. + width.
TK_API int tk_sum_columns(int dtype, const void* in, int parts, long part_stride, long ld, int col0, void* out, int N, int width,
                          hipStream_t stream) {
  if (N <= 0 || width <= 0) return 0;
  if (parts < 1 || col0 < 0 || ld < (long)col0 + width) return -1;
  const RowsIn r{in, 1, parts, part_stride};
  const long total = (long)N * width;
  const unsigned blocks = (unsigned)((total + 255) / 256);
  if (dtype == 0) sum_columns_kernel<float><<<blocks, 256, 0, stream>>>(r, ld, col0, (float*)out, width, total);
  else sum_columns_kernel<bf16_t><<<blocks, 256, 0, stream>>>(r, ld, col0, (bf16_t*)out, width, total);
  return launch_status();
}

// proj: [N, ld] in dtype, float32 (in_f32) or float32 partial sums, its columns [q: kv dim | k: kv dim | v: heads vdim |
// b: heads | ...]; up: [N, uld] likewise, its first heads * dim columns the decays' pre-activations.  conv float32
// [2 kv dim + heads vdim, taps]; state float32 [slots, taps - 1, 2 kv dim + heads vdim]; a_log float32 [heads], dt_bias
// float32 [heads * dim]; out float32 [N, 2 kv dim + heads vdim + heads dim + heads rounded up to four].
// max_tokens: the most tokens a request brings to the step.
TK_API int tk_delta_inputs(int dtype, const void* proj, int in_f32, int parts, long part_stride, long ld, const void* up,
                           int up_f32, int up_parts, long up_stride, long uld, const float* conv, float* state,
                           const float* a_log, const float* dt_bias, const int* q_start, const int* state_slots,
                           float* out, int R, int heads, int kv, int dim, int vdim, int taps, float q_scale,
                           int max_tokens, hipStream_t stream) {
  if (R <= 0 || max_tokens <= 0) return 0;
  const DeltaShape sh{heads, kv, dim, vdim, taps};
  if (heads < 1 || kv < 1 || heads % kv != 0 || dim < 1 || dim > 512 || vdim < 1 || taps < 1 || taps > kMaxTaps ||
      (taps > 1 && state == nullptr) || parts < 1 || (parts > 1 && !in_f32) || up_parts < 1 || (up_parts > 1 && !up_f32) ||
      ld < (long)sh.conv_channels() + heads || uld < (long)heads * dim)
    return -1;
  const RowsIn p{proj, in_f32 || dtype == 0, parts, part_stride}, u{up, up_f32 || dtype == 0, up_parts, up_stride};
  if (dtype == 0)
    return launch_inputs<float>(p, ld, u, uld, conv, state, a_log, dt_bias, q_start, state_slots, out, R, sh, q_scale,
                                max_tokens, stream);
  return launch_inputs<bf16_t>(p, ld, u, uld, conv, state, a_log, dt_bias, q_start, state_slots, out, R, sh, q_scale,
                               max_tokens, stream);
}

// in: what tk_delta_inputs left; state float32 [slots, heads, vdim, dim rounded up to 4]; y float32 [N, heads * vdim].
TK_API int tk_delta_scan(const float* in, float* state, const int* q_start, const int* state_slots, float* y, int R,
                         int heads, int kv, int dim, int vdim, hipStream_t stream) {
  if (R <= 0) return 0;
  if (heads < 1 || heads > 65535 || kv < 1 || heads % kv != 0 || dim < 1 || dim > 512 || vdim < 1) return -1;
  const DeltaShape sh{heads, kv, dim, vdim, 1};
  const dim3 grid(R, heads, (vdim + kColumns - 1) / kColumns);
  if (grid.z > 65535) return -1;
  const bool wide = dim % 4 == 0 && vdim % 4 == 0 && (uintptr_t)in % 16 == 0;
#define TK_DS(PIECES, TB)                                                                                              \
  {                                                                                                                    \
    if (wide) delta_scan_kernel<PIECES, TB, true><<<grid, kScanThreads, 0, stream>>>(in, state, q_start, state_slots, y, sh); \
    else delta_scan_kernel<PIECES, TB, false><<<grid, kScanThreads, 0, stream>>>(in, state, q_start, state_slots, y, sh);     \
  }
  if (dim <= 64) TK_DS(1, 16)
  else if (dim <= 128) TK_DS(2, 16)
  else if (dim <= 192) TK_DS(3, 8)
  else if (dim <= 256) TK_DS(4, 8)
  else TK_DS(8, 4)
#undef TK_DS
  return launch_status();
}

TK_SLOTS(tk_sum_columns)
TK_SLOTS(tk_delta_inputs)
TK_SLOTS(tk_delta_scan)
