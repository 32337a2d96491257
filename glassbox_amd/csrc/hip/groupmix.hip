// Kernels around a sublayer whose input is a grouped RMS norm of the residual plus a short convolution of it over time,
// in a model whose layers hand on weighted sums of everything before them.
//
//   embed_sinusoid  x = table[id] * scale + the position's sine and cosine: channels 2i and 2i + 1 of position p get sin and
//                   cos of p * base^(-2i / d).
//   residual_rows   one pass over the rows of the residual x (float32 [n, d]) that may, in this order:
//                   add a sublayer's result into x, given in the slices that a product which divides k leaves;
//                   form out = sum_j coef[j] hist[j] + coef[count] x of the rows before it (a sum over depth);
//                   norm the result in groups: with d / groups channels a group, each divided by sqrt(mean square + eps),
//                   either as one factor a (row, group) for the kernel after this one, or as rows h = normed * gamma in the
//                   activations' type, and these (a step of single tokens) with their convolution over time added and the
//                   request's slot moved on.
//   norm_conv       h = g + conv(g), g = x * factor * gamma, conv(g)[t] = sum_j w[j] g[t - taps + 1 + j] over the request's own
//                   tokens (zeros before its first); norm_conv_state moves the slots on afterwards.
//
// The residual, the sums, the norms, the convolutions and their state are 32-bit; a value is rounded once, when it is stored
// in the activations' type.
#include "common.h"

using namespace gb;

GB_DEFINE_LAST_ERROR

namespace {

constexpr int kMaxTaps = 8;
constexpr int kMaxGroups = 64;
constexpr int kMaxWide = 8192;     // the widest row kept in registers
constexpr int kMaxAny = 12288;     // the widest row kept in LDS

__device__ __forceinline__ f32x4 load4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ void store4(float* p, const f32x4& v) { *reinterpret_cast<f32x4*>(p) = v; }
__device__ __forceinline__ void store4(bf16* p, const f32x4& v) {
  bf16x4 o;
#pragma unroll
  for (int e = 0; e < 4; ++e) o[e] = (bf16)v[e];
  *reinterpret_cast<bf16x4*>(p) = o;
}
inline bool words16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

// ------------------------------------------------------------------------------------------------ embed_sinusoid
// The angle is a product in 64-bit whose whole turns are dropped before sine and cosine are taken in 32-bit.
template <typename T>
__global__ void embed_sinusoid_kernel(const T* __restrict__ table, const int32_t* __restrict__ ids,
                                      const int32_t* __restrict__ positions, const double* __restrict__ turns, float* __restrict__ x,
                                      int n, int d, int vocab, float scale, int copies) {
  const int i = blockIdx.y, pair = blockIdx.x * blockDim.x + threadIdx.x, c = 2 * pair;
  if (c >= d) return;
  const int id = ids[i];
  const bool ok = id >= 0 && id < vocab;
  const T* row = table + (size_t)(ok ? id : 0) * d;
  double part = (double)positions[i] * turns[pair];   // base^(-2i / d) / (2 pi): turns a position
  part -= rint(part);
  const float ang = (float)(part * 6.283185307179586476925);
  float s, co;
  sincosf(ang, &s, &co);
  const float bad = __builtin_nanf("");               // a bad id must not pass silently
  const float a = ok ? fmaf(to_f(row[c]), scale, s) : bad;
  for (int k = 0; k < copies; ++k) x[((size_t)k * n + i) * d + c] = a;
  if (c + 1 < d) {
    const float b = ok ? fmaf(to_f(row[c + 1]), scale, co) : bad;
    for (int k = 0; k < copies; ++k) x[((size_t)k * n + i) * d + c + 1] = b;
  }
}

// ------------------------------------------------------------------------------------------------ residual_rows
struct RowPass {
  float* x;
  const float* y;              // a sublayer's result in `slices` pieces, or nullptr
  int slices;
  long long slice_stride;
  const float* hist;           // count rows sets of [n, d], hist_stride apart
  long long hist_stride;
  const float* coef;           // [count + 1]
  int count;                   // 0: no sum over depth
  float* out;                  // where that sum goes
  const int32_t* rows;         // picked rows of x (no y, no sum then)
  const float* gamma;
  int groups;                  // 0: no norm
  float eps;
  float* scales;               // [n, groups], or nullptr
  const float* conv_w;         // [taps, d], or nullptr
  int taps;
  float* state;
  long long slot_stride;
  const int32_t *tok_seq, *pos0, *state_slots;
};

// Sums of squares of the groups from the quads' sums in `part` (d / 4 of them, gq a group): a wave a group; leaves the
// groups' factors in `inv`.  The order of the additions is fixed by d and groups alone.
__device__ __forceinline__ void group_factors(const float* part, float* inv, int groups, int gq, float eps) {
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, waves = blockDim.x / kWave;
  for (int g = wave; g < groups; g += waves) {
    float s = 0.f;
    for (int q = lane; q < gq; q += kWave) s += part[g * gq + q];
    s = wave_sum(s);
    if (lane == 0) inv[g] = 1.0f / sqrtf(s / (float)(gq * 4) + eps);
  }
}

// Rows in registers: d and d / groups multiples of 4, d at most THREADS * WORDS * 4.
template <typename T, int THREADS, int WORDS>
__global__ __launch_bounds__(THREADS) void residual_rows_kernel(RowPass p, T* __restrict__ h, int d) {
  __shared__ float part[THREADS * WORDS];
  __shared__ float inv[kMaxGroups];
  const int t = blockIdx.x;
  float* xr = p.x + (size_t)(p.rows ? p.rows[t] : t) * d;
  f32x4 v[WORDS];
  const int K = p.taps - 1;
  int pos = 0;
  float* st = nullptr;
  if (p.conv_w && K > 0) {
    const int seq = p.tok_seq[t];
    pos = p.pos0[seq];
    st = p.state + (size_t)p.state_slots[seq] * p.slot_stride;
  }
  // a step of single tokens is a few of these workgroups, whose time is round trips to memory: what the convolution reads (up
  // to four taps) is on its way from the start
  constexpr int AHEAD = WORDS == 1 ? 4 : 0;
  f32x4 ahead_w[AHEAD > 0 ? AHEAD : 1], ahead_s[AHEAD > 0 ? AHEAD : 1];
  const bool ahead = AHEAD > 0 && p.conv_w && p.taps <= AHEAD && 4 * (int)threadIdx.x < d;
  if (AHEAD > 0 && ahead) {
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      if (j < p.taps) ahead_w[j] = load4(p.conv_w + (size_t)j * d + 4 * threadIdx.x);
      if (j < K) ahead_s[j] = load4(st + (size_t)j * d + 4 * threadIdx.x);
    }
  }
#pragma unroll
  for (int i = 0; i < WORDS; ++i) {
    const int c = (threadIdx.x + i * THREADS) * 4;
    if (c >= d) continue;
    v[i] = load4(xr + c);
    if (p.y) {
      f32x4 s = load4(p.y + (size_t)t * d + c);
      for (int z = 1; z < p.slices; ++z) s += load4(p.y + (size_t)z * p.slice_stride + (size_t)t * d + c);
      v[i] += s;
      store4(xr + c, v[i]);
    }
  }
  if (p.count > 0) {
    f32x4 acc[WORDS];
#pragma unroll
    for (int i = 0; i < WORDS; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll(WORDS == 1 ? 8 : 4)
    for (int j = 0; j < p.count; ++j) {
      const float a = p.coef[j];
      const float* hr = p.hist + (size_t)j * p.hist_stride + (size_t)t * d;
#pragma unroll
      for (int i = 0; i < WORDS; ++i) {
        const int c = (threadIdx.x + i * THREADS) * 4;
        if (c >= d) continue;
        const f32x4 o = load4(hr + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[i][e] = fmaf(a, o[e], acc[i][e]);
      }
    }
    const float a = p.coef[p.count];
#pragma unroll
    for (int i = 0; i < WORDS; ++i) {
      const int c = (threadIdx.x + i * THREADS) * 4;
      if (c >= d) continue;
#pragma unroll
      for (int e = 0; e < 4; ++e) v[i][e] = fmaf(a, v[i][e], acc[i][e]);
      store4(p.out + (size_t)t * d + c, v[i]);
    }
  }
  if (p.groups == 0) return;
#pragma unroll
  for (int i = 0; i < WORDS; ++i) {
    const int q = threadIdx.x + i * THREADS;
    if (4 * q < d) part[q] = (v[i][0] * v[i][0] + v[i][1] * v[i][1]) + (v[i][2] * v[i][2] + v[i][3] * v[i][3]);
  }
  __syncthreads();
  const int gq = d / 4 / p.groups;
  group_factors(part, inv, p.groups, gq, p.eps);
  __syncthreads();
  if (p.scales && (int)threadIdx.x < p.groups) p.scales[(size_t)t * p.groups + threadIdx.x] = inv[threadIdx.x];
  if (!h) return;
#pragma unroll
  for (int i = 0; i < WORDS; ++i) {
    const int q = threadIdx.x + i * THREADS, c = 4 * q;
    if (c >= d) continue;
    const float r = inv[q / gq];
    const f32x4 g = load4(p.gamma + c);
    f32x4 cur;
#pragma unroll
    for (int e = 0; e < 4; ++e) cur[e] = v[i][e] * r * g[e];
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    // index j of the slot is the row of position pos - (K - j); it moves to index j - 1
    auto tap = [&](int j, f32x4 in, const f32x4& wj) {
      if (j < K) {
        if (j > 0) store4(st + (size_t)(j - 1) * d + c, in);
        if (pos - (K - j) < 0) in = f32x4{0.f, 0.f, 0.f, 0.f};   // before the request's first token
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[e] = fmaf(wj[e], in[e], acc[e]);
    };
    if (AHEAD > 0 && ahead) {
#pragma unroll
      for (int j = 0; j < AHEAD; ++j)
        if (j < p.taps) tap(j, j < K ? ahead_s[j] : cur, ahead_w[j]);
    } else if (p.conv_w) {
      for (int j = 0; j < p.taps; ++j) tap(j, j < K ? load4(st + (size_t)j * d + c) : cur, load4(p.conv_w + (size_t)j * d + c));
    }
    if (p.conv_w && K > 0) store4(st + (size_t)(K - 1) * d + c, cur);
    store4(h + (size_t)t * d + c, cur + acc);
  }
}

// Any row up to kMaxAny columns, in LDS: `row` [d], then the groups' factors.
template <typename T>
__global__ __launch_bounds__(256) void residual_rows_any_kernel(RowPass p, T* __restrict__ h, int d) {
  extern __shared__ float row[];
  __shared__ float inv[kMaxGroups];
  const int t = blockIdx.x, tid = threadIdx.x;
  float* xr = p.x + (size_t)(p.rows ? p.rows[t] : t) * d;
  for (int c = tid; c < d; c += 256) {
    float v = xr[c];
    if (p.y) {
      float s = p.y[(size_t)t * d + c];
      for (int z = 1; z < p.slices; ++z) s += p.y[(size_t)z * p.slice_stride + (size_t)t * d + c];
      v += s;
      xr[c] = v;
    }
    if (p.count > 0) {
      float acc = 0.f;
      for (int j = 0; j < p.count; ++j) acc = fmaf(p.coef[j], p.hist[(size_t)j * p.hist_stride + (size_t)t * d + c], acc);
      v = fmaf(p.coef[p.count], v, acc);
      p.out[(size_t)t * d + c] = v;
    }
    row[c] = v;
  }
  if (p.groups == 0) return;
  __syncthreads();
  const int gd = d / p.groups, lane = tid % kWave, wave = tid / kWave;
  for (int g = wave; g < p.groups; g += 4) {
    float s = 0.f;
    for (int c = lane; c < gd; c += kWave) s = fmaf(row[g * gd + c], row[g * gd + c], s);
    s = wave_sum(s);
    if (lane == 0) inv[g] = 1.0f / sqrtf(s / (float)gd + p.eps);
  }
  __syncthreads();
  if (p.scales && tid < p.groups) p.scales[(size_t)t * p.groups + tid] = inv[tid];
  if (!h) return;
  const int K = p.taps - 1;
  int pos = 0;
  float* st = nullptr;
  if (p.conv_w && K > 0) {
    const int seq = p.tok_seq[t];
    pos = p.pos0[seq];
    st = p.state + (size_t)p.state_slots[seq] * p.slot_stride;
  }
  for (int c = tid; c < d; c += 256) {
    const float cur = row[c] * inv[c / gd] * p.gamma[c];
    float acc = 0.f;
    if (p.conv_w) {
      for (int j = 0; j < p.taps; ++j) {
        float in = cur;
        if (j < K) {
          in = st[(size_t)j * d + c];
          if (j > 0) st[(size_t)(j - 1) * d + c] = in;
          if (pos - (K - j) < 0) in = 0.f;
        }
        acc = fmaf(p.conv_w[(size_t)j * d + c], in, acc);
      }
      if (K > 0) st[(size_t)(K - 1) * d + c] = cur;
    }
    h[(size_t)t * d + c] = from_f<T>(cur + acc);
  }
}

// ------------------------------------------------------------------------------------------------ norm_conv
// A thread a (token, channel).
template <typename T>
__global__ void norm_conv_kernel(const float* __restrict__ x, const float* __restrict__ scales, int groups,
                                 const float* __restrict__ gamma, const float* __restrict__ w, int taps,
                                 const float* __restrict__ state, long long slot_stride, const int32_t* __restrict__ tok_seq,
                                 const int32_t* __restrict__ q_start, const int32_t* __restrict__ pos0,
                                 const int32_t* __restrict__ state_slots, T* __restrict__ out, long long count, int d) {
  const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= count) return;
  const int t = (int)(idx / d), c = (int)(idx % d), g = c / (d / groups);
  auto normed = [&](int row) { return x[(size_t)row * d + c] * scales[(size_t)row * groups + g] * gamma[c]; };
  const float cur = normed(t);
  float acc = 0.f;
  if (taps > 0) {
    const int K = taps - 1, seq = tok_seq[t], off = t - q_start[seq], first_pos = pos0[seq];
    const float* st = K > 0 ? state + (size_t)state_slots[seq] * slot_stride + c : nullptr;
    for (int j = 0; j < taps; ++j) {
      const int back = K - j;   // how many tokens before this one
      float v = 0.f;
      if (back == 0) v = cur;
      else if (off >= back) v = normed(t - back);
      else if (first_pos + off - back >= 0) v = st[(size_t)(off + j) * d];   // index (position - back) - first_pos + K
      acc = fmaf(w[(size_t)j * d + c], v, acc);
    }
  }
  out[idx] = from_f<T>(cur + acc);
}

// Four channels and four tokens in a row a thread, so that a row of x is read for four tokens' sums: d and d / groups are
// multiples of 4.  The tokens may be of different requests; each looks up its own.
constexpr int kConvTokens = 4;
template <typename T>
__global__ __launch_bounds__(256) void norm_conv4x4_kernel(const float* __restrict__ x, const float* __restrict__ scales, int groups,
                                                           const float* __restrict__ gamma, const float* __restrict__ w, int taps,
                                                           const float* __restrict__ state, long long slot_stride,
                                                           const int32_t* __restrict__ tok_seq, const int32_t* __restrict__ q_start,
                                                           const int32_t* __restrict__ pos0, const int32_t* __restrict__ state_slots,
                                                           T* __restrict__ out, int n, int d) {
  const int t0 = blockIdx.x * kConvTokens, c = (blockIdx.y * 256 + threadIdx.x) * 4;
  if (c >= d) return;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  const int K = taps > 0 ? taps - 1 : 0, g = c / (d / groups);
  // rows[k] is token t0 - K + k: what the four tokens' taps can reach of the step's rows; tap j of token t0 + i reads
  // rows[i + j]
  f32x4 rows[kMaxTaps - 1 + kConvTokens], wv[kMaxTaps];
  float sc[kMaxTaps - 1 + kConvTokens];
  const f32x4 gm = load4(gamma + c);
#pragma unroll
  for (int k = 0; k < kMaxTaps - 1 + kConvTokens; ++k) {
    const int t = t0 - K + k;
    const bool there = k < K + kConvTokens && t >= 0 && t < n;
    rows[k] = there ? load4(x + (size_t)t * d + c) : zero;
    sc[k] = there ? scales[(size_t)t * groups + g] : 0.f;
  }
#pragma unroll
  for (int j = 0; j < kMaxTaps; ++j) wv[j] = j < taps ? load4(w + (size_t)j * d + c) : zero;
#pragma unroll
  for (int k = 0; k < kMaxTaps - 1 + kConvTokens; ++k)
#pragma unroll
    for (int e = 0; e < 4; ++e) rows[k][e] = rows[k][e] * sc[k] * gm[e];
#pragma unroll
  for (int i = 0; i < kConvTokens; ++i) {
    const int t = t0 + i;
    if (t >= n) break;
    f32x4 acc = zero, cur = zero;
    // (the token's own row is rows[i + K]: an index the compiler must know)
#pragma unroll
    for (int k = 0; k < kMaxTaps; ++k)
      if (k == K) cur = rows[i + k];
    if (taps > 0) {
      const int seq = tok_seq[t], off = t - q_start[seq], first_pos = pos0[seq];
      const float* st = K > 0 ? state + (size_t)state_slots[seq] * slot_stride + c : nullptr;
#pragma unroll
      for (int j = 0; j < kMaxTaps; ++j) {
        if (j >= taps) break;
        const int back = K - j;
        f32x4 v = zero;
        if (off >= back) v = rows[i + j];
        else if (first_pos + off - back >= 0) v = load4(st + (size_t)(off + j) * d);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[e] = fmaf(wv[j][e], v[e], acc[e]);
      }
    }
    store4(out + (size_t)t * d + c, cur + acc);
  }
}

// A thread a (request, channel): the slot's taps - 1 rows become the request's last ones.
__global__ void norm_conv_state_kernel(const float* __restrict__ x, const float* __restrict__ scales, int groups,
                                       const float* __restrict__ gamma, float* __restrict__ state, long long slot_stride,
                                       const int32_t* __restrict__ q_start, const int32_t* __restrict__ q_len,
                                       const int32_t* __restrict__ state_slots, int d, int taps) {
  const int seq = blockIdx.y, c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= d) return;
  const int L = q_len[seq], start = q_start[seq], K = taps - 1, g = c / (d / groups);
  float* st = state + (size_t)state_slots[seq] * slot_stride + c;
  float nv[kMaxTaps - 1];
#pragma unroll
  for (int i = 0; i < kMaxTaps - 1; ++i) {
    nv[i] = 0.f;
    if (i < K) {
      const int r = L - K + i;   // the step's row that lands here, if there is one
      const size_t row = (size_t)(start + r);
      nv[i] = r >= 0 ? x[row * d + c] * scales[row * groups + g] * gamma[c] : st[(size_t)(i + L) * d];
    }
  }
#pragma unroll
  for (int i = 0; i < kMaxTaps - 1; ++i)
    if (i < K) st[(size_t)i * d] = nv[i];
}

inline bool grid_fits(long long count, int per_block) { return (count + per_block - 1) / per_block < (1ll << 31); }

}  // namespace

#define GB_BY_DTYPE(dtype, what, CALL)              \
  if (dtype == kF32) {                              \
    typedef float TT;                               \
    CALL;                                           \
  } else if (dtype == kBF16) {                      \
    typedef bf16 TT;                                \
    CALL;                                           \
  } else {                                          \
    return fail(what ": unknown dtype %d", dtype);  \
  }

// table [vocab, d], ids and positions [n], turns float64 [ceil(d / 2)], x float32 [copies, n, d].
extern "C" int gb_embed_sinusoid(const void* table, int table_dtype, const int32_t* ids, const int32_t* positions,
                                 const double* turns, float* x, int n, int d, int vocab, float scale, int copies,
                                 hipStream_t stream) {
  GB_REQUIRE(n >= 0 && d > 0 && vocab > 0 && copies > 0 && ids && positions && turns, "embed_sinusoid: bad sizes n=%d d=%d vocab=%d copies=%d", n, d, vocab, copies);
  if (n == 0) return 0;
  const int pairs = (d + 1) / 2;
  for (int first = 0; first < n; first += 65535) {   // a launch takes 65,535 rows; the copies keep their distance of n rows
    const int rows = n - first < 65535 ? n - first : 65535;
    const dim3 grid((unsigned)((pairs + 255) / 256), (unsigned)rows);
    GB_REQUIRE(copies == 1 || rows == n, "embed_sinusoid: several copies of more than 65535 rows");
    GB_BY_DTYPE(table_dtype, "embed_sinusoid",
                hipLaunchKernelGGL(embed_sinusoid_kernel<TT>, grid, dim3(256), 0, stream, (const TT*)table, ids + first,
                                   positions + first, turns, x + (size_t)first * d, n, d, vocab, scale, copies))
  }
  return launched("embed_sinusoid");
}

// x float32 [*, d].  y (or nullptr): float32, `slices` pieces of [n, d], added into x.  count > 0: out [n, d] receives
// sum_j coef[j] hist[j] + coef[count] x (hist: count pieces of [n, d], hist_stride apart).  groups > 0: the grouped norm of
// the result: factors to scales [n, groups] and / or rows to h [n, d] of `dtype` (with gamma [d]); conv_w [taps, d] (a step in
// which every request brings one row): h receives rows + conv(rows), and the slots (slot_stride floats apart, [taps - 1, d]
// each) are moved on.  rows (or nullptr): row t of the result is row rows[t] of x (norm only).
extern "C" int gb_residual_rows(float* x, const float* y, int slices, long long slice_stride, const float* hist,
                                long long hist_stride, const float* coef, int count, float* out, const int32_t* rows,
                                const float* gamma, int groups, float eps, float* scales, void* h, int dtype, const float* conv_w,
                                int taps, float* state, long long slot_stride, const int32_t* tok_seq, const int32_t* pos0,
                                const int32_t* state_slots, int n, int d, hipStream_t stream) {
  GB_REQUIRE(n >= 0 && d > 0 && x, "residual_rows: bad sizes n=%d d=%d", n, d);
  GB_REQUIRE(!y || (slices >= 1 && (slices == 1 || slice_stride >= (long long)n * d)), "residual_rows: %d slices", slices);
  GB_REQUIRE(count >= 0 && (count == 0 || (hist && coef && out && hist_stride >= (long long)n * d)), "residual_rows: a sum over %d rows before this one needs them", count);
  GB_REQUIRE(groups >= 0 && groups <= kMaxGroups && (groups == 0 || d % groups == 0), "residual_rows: %d groups of %d columns (at most %d)", groups, d, kMaxGroups);
  GB_REQUIRE(groups > 0 || (!scales && !h), "residual_rows: a norm's result without its groups");
  GB_REQUIRE(!h || gamma, "residual_rows: normed rows need their weight");
  GB_REQUIRE(!rows || (!y && count == 0 && !conv_w), "residual_rows: picked rows are only normed");
  GB_REQUIRE(!conv_w || (h && taps >= 1 && taps <= kMaxTaps && tok_seq && pos0 && state_slots && (taps == 1 || (state && slot_stride >= (long long)(taps - 1) * d))),
             "residual_rows: the convolution needs a result, weights of at most %d taps, the step's tables and the state", kMaxTaps);
  if (n == 0) return 0;
  const RowPass p{x, y, slices, slice_stride, hist, hist_stride, coef, count, out, rows, gamma, groups, eps, scales,
                  conv_w, conv_w ? taps : 0, state, slot_stride, tok_seq, pos0, state_slots};
  const bool words = d % 4 == 0 && (groups == 0 || d / groups % 4 == 0) && d <= kMaxWide && words16(x) && words16(y) && words16(hist) &&
                     words16(out) && words16(h) && words16(gamma) && words16(conv_w) && words16(state) && slice_stride % 4 == 0 &&
                     hist_stride % 4 == 0 && slot_stride % 4 == 0;
  if (words) {
    const int quads = d / 4;
#define GB_ROWS(THREADS, WORDS)                                                                                              \
  GB_BY_DTYPE(dtype, "residual_rows",                                                                                          \
              hipLaunchKernelGGL((residual_rows_kernel<TT, THREADS, WORDS>), dim3((unsigned)n), dim3(THREADS), 0, stream, p, (TT*)h, d))
    if (n >= 512) {
      if (quads <= 256) { GB_ROWS(256, 1) } else if (quads <= 512) { GB_ROWS(256, 2) } else if (quads <= 1024) { GB_ROWS(256, 4) } else { GB_ROWS(256, 8) }
    } else {
      if (quads <= 256) { GB_ROWS(256, 1) } else if (quads <= 512) { GB_ROWS(512, 1) } else if (quads <= 1024) { GB_ROWS(1024, 1) } else { GB_ROWS(1024, 2) }
    }
#undef GB_ROWS
    return launched("residual_rows");
  }
  GB_REQUIRE(d <= kMaxAny, "residual_rows: rows of %d columns (at most %d)", d, kMaxAny);
  GB_BY_DTYPE(dtype, "residual_rows",
              hipLaunchKernelGGL(residual_rows_any_kernel<TT>, dim3((unsigned)n), dim3(256), (size_t)d * sizeof(float), stream, p, (TT*)h, d))
  return launched("residual_rows");
}

// x float32 [n, d], scales float32 [n, groups] (as residual_rows leaves them), gamma [d], w [taps, d] (taps 0: no
// convolution), slots as in gb_residual_rows, out [n, d] of `dtype`.  With taps > 1 the caller moves the slots on after this
// call (gb_norm_conv_state), before x changes.
extern "C" int gb_norm_conv(const float* x, const float* scales, int groups, const float* gamma, const float* w, int taps,
                            const float* state, long long slot_stride, const int32_t* tok_seq, const int32_t* q_start,
                            const int32_t* pos0, const int32_t* state_slots, void* out, int dtype, int n, int d,
                            hipStream_t stream) {
  GB_REQUIRE(n >= 0 && d > 0 && groups > 0 && d % groups == 0 && x && scales && gamma && out, "norm_conv: bad sizes n=%d d=%d groups=%d", n, d, groups);
  GB_REQUIRE(taps >= 0 && taps <= kMaxTaps, "norm_conv: %d taps (at most %d)", taps, kMaxTaps);
  GB_REQUIRE(taps == 0 || (w && tok_seq && q_start && pos0 && state_slots && (taps == 1 || (state && slot_stride >= (long long)(taps - 1) * d))),
             "norm_conv: weights, the step's tables and the state are needed");
  if (n == 0) return 0;
  const long long count = (long long)n * d;
  GB_REQUIRE(grid_fits(count, 256), "norm_conv: too many elements");
  if (d % 4 == 0 && d / groups % 4 == 0 && words16(x) && words16(out) && words16(state) && words16(w) && words16(gamma) &&
      slot_stride % 4 == 0 && (d + 1023) / 1024 < 65536) {
    const dim3 grid((unsigned)((n + kConvTokens - 1) / kConvTokens), (unsigned)((d + 1023) / 1024));
    GB_BY_DTYPE(dtype, "norm_conv",
                hipLaunchKernelGGL(norm_conv4x4_kernel<TT>, grid, dim3(256), 0, stream, x, scales, groups, gamma, w, taps, state,
                                   slot_stride, tok_seq, q_start, pos0, state_slots, (TT*)out, n, d))
    return launched("norm_conv");
  }
  GB_BY_DTYPE(dtype, "norm_conv",
              hipLaunchKernelGGL(norm_conv_kernel<TT>, dim3((unsigned)((count + 255) / 256)), dim3(256), 0, stream, x, scales, groups,
                                 gamma, w, taps, state, slot_stride, tok_seq, q_start, pos0, state_slots, (TT*)out, count, d))
  return launched("norm_conv");
}

extern "C" int gb_norm_conv_state(const float* x, const float* scales, int groups, const float* gamma, float* state,
                                  long long slot_stride, const int32_t* q_start, const int32_t* q_len,
                                  const int32_t* state_slots, int n_seqs, int d, int taps, hipStream_t stream) {
  GB_REQUIRE(n_seqs >= 0 && n_seqs <= 65535 && d > 0 && groups > 0 && d % groups == 0 && taps >= 1 && taps <= kMaxTaps,
             "norm_conv_state: bad sizes requests=%d d=%d taps=%d", n_seqs, d, taps);
  if (n_seqs == 0 || taps == 1) return 0;
  GB_REQUIRE(x && scales && gamma && state && q_start && q_len && state_slots && slot_stride >= (long long)(taps - 1) * d, "norm_conv_state: operands are missing");
  hipLaunchKernelGGL(norm_conv_state_kernel, dim3((unsigned)((d + 255) / 256), (unsigned)n_seqs), dim3(256), 0, stream, x, scales,
                     groups, gamma, state, slot_stride, q_start, q_len, state_slots, d, taps);
  return launched("norm_conv_state");
}

// the launches of a layer can be recorded and made again for the layers like it (common.h)
GB_TAPED(gb_embed_sinusoid)
GB_TAPED(gb_residual_rows)
GB_TAPED(gb_norm_conv)
GB_TAPED(gb_norm_conv_state)
