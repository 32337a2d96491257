// The gated delta rule: a decayed matrix state per (request, head) that is corrected towards each token's value.
//
//   S <- diag(g_t) S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t        S: [dk, dv]
//
// H heads of dv value channels share G query/key heads of dk channels (head h uses number h / (H / G)).  q, k and v are the
// projections behind a causal convolution over time and silu; q and k have length one (q also times dk^(-1/2)).  The decay
// is log g = -rate[h] softplus(z + dt), z one number a head and token (`channel` 0) or one a head, key channel and token.
// Everything from the unit lengths on is 32-bit.
//
// A request's slot holds S, 32-bit, [H, dv, dk] (a column of S in a row of memory), and behind it (`ring_at` floats into the
// slot) the convolution's inputs as a ring of `taps` rows of 2 G dk + H dv channels: position p's row is number p % taps.  A
// token reads the rows of the taps - 1 positions before its own and its own projections; it leaves its row at a place that
// no reader of the same step needs, so every workgroup of a single token's step may read the ring while one writes it.
//
// Single tokens: `step` does everything from the projections to the gated heads, a workgroup a (token, head).  Short portions:
// `prep` (convolution, unit lengths, beta, log decays), `scan` (token after token, eight lanes a column, the state in registers),
// `out` (norm and gate).  Long portions go in chunks of 64 tokens.  With G_i the sum of the log decays of the chunk's tokens up to
// i, S0 the state before the chunk and
//   A_ij = beta_i sum_c k_ic k_jc e^(G_ic - G_jc) (j < i),   P_ij = sum_c q_ic k_jc e^(G_ic - G_jc) (j <= i),
// the chunk's corrections are u = (I + A)^(-1) (beta v - (beta e^G k) S0) = U - W S0, its outputs
// (e^G q) S0 + P u = (e^G q - P W) S0 + P U, and the state behind it e^(G_last) S0 + (e^(G_last - G) k)^T u = M S0 + B with
// M = diag(e^(G_last)) - (e^(G_last - G) k)^T W and B = (e^(G_last - G) k)^T U.  `chunk` makes Q' = e^G q - P W, O' = P U, M and B of all
// chunks side by side, from the projections; `chain` walks a request's chunks, S <- M S + B, which is all that waits for the
// chunk before, and leaves the state before each; `emit` makes Q' S0 + O', normed and gated, of all chunks side by side.  All
// products are 32-bit (v_mfma_f32_16x16x4_f32).  No exponent above zero is ever taken: A and P fall into blocks of 16 x 16; off the
// diagonal both factors decay from or to the last token before the block row, and on the diagonal each pair's factor is the
// running product of the decays between its tokens.
#include "common.h"

using namespace gb;

GB_DEFINE_LAST_ERROR

namespace {

constexpr int kMaxTaps = 8;
constexpr int kLanesCol = 8;   // lanes a column of the state
constexpr int kC = 64;         // tokens a chunk

// What every kernel knows of a step's requests and of the state.
struct Rows {
  const int32_t* __restrict__ tok_seq;
  const int32_t* __restrict__ q_start;
  const int32_t* __restrict__ q_len;
  const int32_t* __restrict__ pos0;
  const int32_t* __restrict__ slots;
  float* __restrict__ state;
  long long slot_floats, ring_at;
};
struct Sizes {
  int H, G, dk, dv, taps;
};
// The projections' columns: q, k, v side by side from `at` on; beta's and (channel 0) the decay's logits a head.
struct Proj {
  int ld, at, b_at, a_at;
};
// The decay's constants, and with channel != 0 its logits [n, ldz] in 32-bit.
struct Decay {
  const float* __restrict__ rate;   // [H]
  const float* __restrict__ dt;     // [H], or [H dk]
  const float* __restrict__ z;
  int ldz, channel;
};

// Sum over the eight lanes of a column (lanes 8c .. 8c+7), by moves inside the wave's rows of 16 lanes.
__device__ __forceinline__ float sum8(float v) {
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xf, 0xf, false));   // quad_perm [1,0,3,2]
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x4E, 0xf, 0xf, false));   // quad_perm [2,3,0,1]
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x141, 0xf, 0xf, false));  // row_half_mirror
  return v;
}
__device__ __forceinline__ float sum16(float v) {
#pragma unroll
  for (int o = 1; o < 16; o <<= 1) v += __shfl_xor(v, o, kWave);
  return v;
}
// Exponentials, logarithms and reciprocals by the hardware's instructions (an ulp each, in units of log2).
constexpr float kLog2e = 1.4426950408889634f, kLn2 = 0.6931471805599453f;
__device__ __forceinline__ float exp2_of(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float exp_of(float x) { return exp2_of(x * kLog2e); }
__device__ __forceinline__ float sigmoid(float x) { return __builtin_amdgcn_rcpf(1.0f + exp_of(-x)); }
__device__ __forceinline__ float silu(float x) { return x * sigmoid(x); }
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.f) + kLn2 * __builtin_amdgcn_logf(1.0f + exp_of(-fabsf(x))); }

// The convolved channel ch (0 .. 2 G dk + H dv - 1) of step row t, which is token `off` of its request's rows and at
// position `pos`; ring: the request's ring.
template <typename T>
__device__ __forceinline__ float convolved(const T* __restrict__ proj, const Proj& p, const float* __restrict__ wconv, int taps,
                                           int channels, int ch, int t, int off, int pos, const float* __restrict__ ring) {
  float acc = 0.f;
  for (int j = 0; j < taps; ++j) {
    const int back = taps - 1 - j;
    float x = 0.f;
    if (off >= back) x = to_f(proj[(size_t)(t - back) * p.ld + p.at + ch]);
    else if (pos - back >= 0) x = ring[(size_t)((pos - back) % taps) * channels + ch];
    acc = fmaf(wconv[(size_t)j * channels + ch], x, acc);
  }
  return acc;
}
// The same for four neighbouring channels (whole words).
template <typename T>
__device__ __forceinline__ f32x4 convolved4(const T* __restrict__ proj, const Proj& p, const float* __restrict__ wconv, int taps,
                                            int channels, int ch, int t, int off, int pos, const float* __restrict__ ring) {
  typedef T quad __attribute__((ext_vector_type(4)));
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int j = 0; j < taps; ++j) {
    const int back = taps - 1 - j;
    f32x4 x = {0.f, 0.f, 0.f, 0.f};
    if (off >= back) {
      const quad w = *reinterpret_cast<const quad*>(proj + (size_t)(t - back) * p.ld + p.at + ch);
#pragma unroll
      for (int e = 0; e < 4; ++e) x[e] = to_f(w[e]);
    } else if (pos - back >= 0) {
      x = *reinterpret_cast<const f32x4*>(ring + (size_t)((pos - back) % taps) * channels + ch);
    }
    const f32x4 wt = *reinterpret_cast<const f32x4*>(wconv + (size_t)j * channels + ch);
#pragma unroll
    for (int e = 0; e < 4; ++e) acc[e] = fmaf(wt[e], x[e], acc[e]);
  }
  return acc;
}

// The same where every input is one of the step's rows, none of them before row t_min: no branches, so that all loads of a caller's
// several calls are on their way together.  MT >= taps: the surplus reads an input again and counts it zero times.
template <typename T, int MT>
__device__ __forceinline__ f32x4 convolved4_rows(const T* __restrict__ proj, const Proj& p, const float* __restrict__ wconv, int taps,
                                                 int channels, int ch, int t, int t_min) {
  typedef T quad __attribute__((ext_vector_type(4)));
  quad x[MT];
  f32x4 w[MT];
#pragma unroll
  for (int b = 0; b < MT; ++b) {
    const int back = min(b, taps - 1);
    x[b] = *reinterpret_cast<const quad*>(proj + (size_t)max(t - back, t_min) * p.ld + p.at + ch);
    w[b] = *reinterpret_cast<const f32x4*>(wconv + (size_t)(taps - 1 - back) * channels + ch);
  }
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int b = MT - 1; b >= 0; --b) {   // (the oldest first, as elsewhere)
    const bool counts = b < taps;
#pragma unroll
    for (int e = 0; e < 4; ++e) acc[e] = counts ? fmaf(w[b][e], to_f(x[b][e]), acc[e]) : acc[e];
  }
  return acc;
}

// ------------------------------------------------------------------------------------------------ prep
// q32, k32 [n, G dk], v [n, H dv], beta [n, H] and lg [n, H] or [n, H dk] of rows first .. first + n - 1 of the step (all
// arrays are indexed by the step's row).  Sixteen lanes a (row, head); units of a row: G query heads, G key heads, H value
// heads, then one for the betas and (channel 0) decays, or (channel) H for the decays of a head each and the betas.
template <typename T, bool WORDS>
__global__ __launch_bounds__(256) void prep_kernel(const T* __restrict__ proj, Proj p, const float* __restrict__ wconv, Decay dc,
                                                   Rows rw, Sizes sz, int first, int n, float* __restrict__ q32,
                                                   float* __restrict__ k32, T* __restrict__ v, float* __restrict__ beta,
                                                   float* __restrict__ lg, int units, float q_scale) {
  typedef T quad __attribute__((ext_vector_type(4)));
  const long long group = (long long)blockIdx.x * 16 + threadIdx.x / 16;
  const int li = threadIdx.x % 16;
  if (group >= (long long)n * units) return;   // (a group of sixteen lanes as a whole; the shuffles below stay inside it)
  const int t = first + (int)(group / units), u = (int)(group % units);
  const int H = sz.H, G = sz.G, dk = sz.dk, dv = sz.dv, channels = 2 * G * dk + H * dv;
  if (u >= 2 * G + H) {
    const T* row = proj + (size_t)t * p.ld;
    if (dc.channel) {
      const int h = u - 2 * G - H;
      const float rate = dc.rate[h];
      for (int c = li; c < dk; c += 16)
        lg[((size_t)t * H + h) * dk + c] = -rate * softplus(dc.z[(size_t)t * dc.ldz + h * dk + c] + dc.dt[h * dk + c]);
      if (li == 0) beta[(size_t)t * H + h] = sigmoid(to_f(row[p.b_at + h]));
    } else {
      for (int h = li; h < H; h += 16) {
        beta[(size_t)t * H + h] = sigmoid(to_f(row[p.b_at + h]));
        lg[(size_t)t * H + h] = -dc.rate[h] * softplus(to_f(row[p.a_at + h]) + dc.dt[h]);
      }
    }
    return;
  }
  const int seq = rw.tok_seq[t], off = t - rw.q_start[seq], pos = rw.pos0[seq] + off;
  const float* ring = rw.state + (size_t)rw.slots[seq] * rw.slot_floats + rw.ring_at;
  const bool is_v = u >= 2 * G;
  const int size = is_v ? dv : dk, ch0 = is_v ? 2 * G * dk + (u - 2 * G) * dv : u * dk;
  if (is_v) {
    T* o = v + (size_t)t * H * dv + (u - 2 * G) * dv;
    if (WORDS) {
      for (int c = li * 4; c < size; c += 64) {
        const f32x4 x = convolved4(proj, p, wconv, sz.taps, channels, ch0 + c, t, off, pos, ring);
        quad y;
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = from_f<T>(silu(x[e]));
        *reinterpret_cast<quad*>(o + c) = y;
      }
    } else {
      for (int c = li; c < size; c += 16) o[c] = from_f<T>(silu(convolved(proj, p, wconv, sz.taps, channels, ch0 + c, t, off, pos, ring)));
    }
    return;
  }
  constexpr int IT = WORDS ? 4 : 16;   // dk <= 256
  float ss = 0.f;
  f32x4 x4[WORDS ? IT : 1];
  float x1[WORDS ? 1 : IT];
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    if constexpr (WORDS) {
      const int c = (i * 16 + li) * 4;
      if (c < size) {
        f32x4 y = convolved4(proj, p, wconv, sz.taps, channels, ch0 + c, t, off, pos, ring);
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = silu(y[e]), ss = fmaf(y[e], y[e], ss);
        x4[i] = y;
      }
    } else {
      const int c = i * 16 + li;
      if (c < size) {
        x1[i] = silu(convolved(proj, p, wconv, sz.taps, channels, ch0 + c, t, off, pos, ring));
        ss = fmaf(x1[i], x1[i], ss);
      }
    }
  }
  const bool is_q = u < G;
  const float s = (is_q ? q_scale : 1.f) / sqrtf(sum16(ss) + 1e-6f);
  float* o = (is_q ? q32 : k32) + (size_t)t * G * dk + (is_q ? u : u - G) * dk;
#pragma unroll
  for (int i = 0; i < IT; ++i) {
    if constexpr (WORDS) {
      const int c = (i * 16 + li) * 4;
      if (c < size) *reinterpret_cast<f32x4*>(o + c) = x4[i] * s;
    } else {
      const int c = i * 16 + li;
      if (c < size) o[c] = x1[i] * s;
    }
  }
}

// The ring after a portion: the rows of its last `taps` positions (older ones are where they were).
template <typename T>
__global__ __launch_bounds__(256) void ring_kernel(const T* __restrict__ proj, Proj p, Rows rw, int taps, int channels, int seq_base) {
  const int seq = seq_base + blockIdx.x, ch = blockIdx.y * 256 + threadIdx.x;
  if (ch >= channels) return;
  const int L = rw.q_len[seq], start = rw.q_start[seq], pos0 = rw.pos0[seq];
  float* ring = rw.state + (size_t)rw.slots[seq] * rw.slot_floats + rw.ring_at;
  for (int i = max(0, L - taps); i < L; ++i)
    ring[(size_t)((pos0 + i) % taps) * channels + ch] = to_f(proj[(size_t)(start + i) * p.ld + p.at + ch]);
}

// ------------------------------------------------------------------------------------------------ scan
// A lane's R rows of its column: words of four, row (m / 4) * 32 + rg * 4 + m % 4 (a column's eight lanes read whole lines).
__device__ __forceinline__ int row_of(int m, int rg) { return (m / 4) * 32 + rg * 4 + m % 4; }

template <int R>
__device__ __forceinline__ void load_column(float (&S)[R], const float* __restrict__ col, int dk, int rg, bool ok) {
#pragma unroll
  for (int m = 0; m < R; m += 4) {
    const int r0 = row_of(m, rg);
    f32x4 w = {0.f, 0.f, 0.f, 0.f};
    if (ok && (dk & 3) == 0) {
      if (r0 < dk) w = *reinterpret_cast<const f32x4*>(col + r0);
    } else if (ok) {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (r0 + e < dk) w[e] = col[r0 + e];
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) S[m + e] = w[e];
  }
}
template <int R>
__device__ __forceinline__ void store_column(const float (&S)[R], float* __restrict__ col, int dk, int rg, bool ok) {
  if (!ok) return;
#pragma unroll
  for (int m = 0; m < R; m += 4) {
    const int r0 = row_of(m, rg);
    if ((dk & 3) == 0) {
      if (r0 < dk) *reinterpret_cast<f32x4*>(col + r0) = f32x4{S[m], S[m + 1], S[m + 2], S[m + 3]};
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (r0 + e < dk) col[r0 + e] = S[m + e];
    }
  }
}

// grid (columns / 32, heads, requests from seq_base on)
template <typename T, int R>
__global__ __launch_bounds__(256) void scan_kernel(const float* __restrict__ q, const float* __restrict__ k, const T* __restrict__ v,
                                                   const float* __restrict__ beta, const float* __restrict__ lg, int channel,
                                                   float* __restrict__ out, Rows rw, Sizes sz, int seq_base) {
  constexpr int DKP = R * kLanesCol, TOK = 8, PER = (TOK * DKP + 255) / 256;
  __shared__ float qs[TOK][DKP], ks[TOK][DKP], gs[TOK][DKP], vs[TOK][32], bs[TOK];
  const int seq = seq_base + blockIdx.z, h = blockIdx.y, col0 = blockIdx.x * 32;
  const int tid = threadIdx.x, rg = tid % kLanesCol, cb = tid / kLanesCol, col = col0 + cb;
  const int H = sz.H, G = sz.G, dk = sz.dk, dv = sz.dv, g = h / (H / G);
  const int first = rw.q_start[seq], count = rw.q_len[seq];
  const bool live = col < dv;
  float* column = rw.state + (size_t)rw.slots[seq] * rw.slot_floats + ((size_t)h * dv + (live ? col : 0)) * dk;
  float S[R];
  load_column<R>(S, column, dk, rg, live && rw.pos0[seq] > 0);
  for (int t0 = 0; t0 < count; t0 += TOK) {
    const int here = min(TOK, count - t0);
    __syncthreads();
#pragma unroll
    for (int e = 0; e < PER; ++e) {
      const int idx = tid + e * 256, tok = idx / DKP, c = idx % DKP;
      if (idx < TOK * DKP) {
        const bool ok = tok < here && c < dk;
        const size_t t = (size_t)(first + t0 + tok);
        qs[tok][c] = ok ? q[t * G * dk + g * dk + c] : 0.f;
        ks[tok][c] = ok ? k[t * G * dk + g * dk + c] : 0.f;
        gs[tok][c] = ok ? exp_of(channel ? lg[(t * H + h) * dk + c] : lg[t * H + h]) : 0.f;
      }
    }
    {
      const int tok = tid / 32, c = tid % 32;
      const size_t t = (size_t)(first + t0 + tok);
      vs[tok][c] = tok < here && col0 + c < dv ? to_f(v[t * H * dv + (size_t)h * dv + col0 + c]) : 0.f;
      if (tid < TOK) bs[tid] = tid < here ? beta[(size_t)(first + t0 + tid) * H + h] : 0.f;
    }
    __syncthreads();
    for (int j = 0; j < here; ++j) {
      float dot = 0.f, o = 0.f;
#pragma unroll
      for (int m = 0; m < R; ++m) {
        S[m] *= gs[j][row_of(m, rg)];
        dot = fmaf(S[m], ks[j][row_of(m, rg)], dot);
      }
      const float u = bs[j] * (vs[j][cb] - sum8(dot));
#pragma unroll
      for (int m = 0; m < R; ++m) {
        S[m] = fmaf(ks[j][row_of(m, rg)], u, S[m]);
        o = fmaf(S[m], qs[j][row_of(m, rg)], o);
      }
      o = sum8(o);
      if (rg == 0 && live) out[(size_t)(first + t0 + j) * H * dv + (size_t)h * dv + col] = o;
    }
  }
  store_column<R>(S, column, dk, rg, live);
}

// ------------------------------------------------------------------------------------------------ step
// out[h] = norm weight * o / sqrt(mean(o^2) + eps) * act(gate), act = silu or (sigmoid_gate) sigmoid.
struct Gate {
  const void* __restrict__ gate;
  int ld, f32, sigmoid;
  const float* __restrict__ w;   // [dv]
  float eps;
  template <typename T> __device__ __forceinline__ float at(size_t row, int col) const {
    const float x = f32 ? static_cast<const float*>(gate)[row * ld + col] : to_f(static_cast<const T*>(gate)[row * ld + col]);
    const float s = __builtin_amdgcn_rcpf(1.0f + exp_of(-x));
    return sigmoid ? s : x * s;
  }
};

// Single tokens: row t of the step is request t's one row.  grid (heads, rows); LDS: 3 DKP + 2 dv + 8 floats.
template <typename T, int R>
__global__ __launch_bounds__(256) void step_kernel(const T* __restrict__ proj, Proj p, const float* __restrict__ wconv, Decay dc,
                                                   Rows rw, Sizes sz, float q_scale, Gate gt, T* __restrict__ out, int ldo) {
  constexpr int DKP = R * kLanesCol;
  extern __shared__ float lds[];
  const int H = sz.H, G = sz.G, dk = sz.dk, dv = sz.dv, taps = sz.taps;
  float *qs = lds, *ks = qs + DKP, *gs = ks + DKP, *vs = gs + DKP, *os = vs + dv, *parts = os + dv;   // parts [8]
  const int h = blockIdx.x, t = blockIdx.y, g = h / (H / G);
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, rg = tid % kLanesCol, cb = tid / kLanesCol;
  const int pos = rw.pos0[t], channels = 2 * G * dk + H * dv;
  float* slot = rw.state + (size_t)rw.slots[t] * rw.slot_floats;
  float* head = slot + (size_t)h * dv * dk;
  float* ring = slot + rw.ring_at;
  const T* row = proj + (size_t)t * p.ld;
  // the first columns of the state are asked for before the convolution's arithmetic
  float S[R];
  load_column<R>(S, head + (size_t)cb * dk, dk, rg, pos > 0 && cb < dv);
  const int own = taps > 1 ? pos % taps : 0;
  if (wave < 2) {   // the query head, the key head: a wave each
    const bool is_q = wave == 0;
    const int ch0 = (is_q ? g : G + g) * dk;
    constexpr int N = (DKP + kWave - 1) / kWave;
    float x[N], ss = 0.f;
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int c = i * kWave + lane;
      x[i] = 0.f;
      if (c < dk) {
        x[i] = silu(convolved(proj, p, wconv, taps, channels, ch0 + c, t, 0, pos, ring));
        // (every head of the group reads the rows of earlier positions; the group's first one leaves this one's)
        if (taps > 1 && h % (H / G) == 0) ring[(size_t)own * channels + ch0 + c] = to_f(row[p.at + ch0 + c]);
      }
      ss = fmaf(x[i], x[i], ss);
    }
    const float s = (is_q ? q_scale : 1.f) / sqrtf(wave_sum(ss) + 1e-6f);
    float* o = is_q ? qs : ks;
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int c = i * kWave + lane;
      if (c < DKP) o[c] = x[i] * s;
    }
  } else if (wave == 2) {
    for (int c = lane; c < dv; c += kWave) {
      const int ch = 2 * G * dk + h * dv + c;
      vs[c] = silu(convolved(proj, p, wconv, taps, channels, ch, t, 0, pos, ring));
      if (taps > 1) ring[(size_t)own * channels + ch] = to_f(row[p.at + ch]);
    }
    if (lane == 0) parts[0] = sigmoid(to_f(row[p.b_at + h]));
  } else {
    const float rate = dc.rate[h];
    const float whole = dc.channel ? 0.f : exp_of(-rate * softplus(to_f(row[p.a_at + h]) + dc.dt[h]));
    for (int c = lane; c < DKP; c += kWave)
      gs[c] = !dc.channel ? whole
              : c < dk    ? exp_of(-rate * softplus(dc.z[(size_t)t * dc.ldz + h * dk + c] + dc.dt[h * dk + c]))
                          : 0.f;
  }
  __syncthreads();
  float qq[R], kk[R], gg[R];
#pragma unroll
  for (int m = 0; m < R; ++m) qq[m] = qs[row_of(m, rg)], kk[m] = ks[row_of(m, rg)], gg[m] = gs[row_of(m, rg)];
  const float beta = parts[0];
  float ss = 0.f;   // of this thread's columns (the first lane of each column counts)
  for (int c0 = 0; c0 < dv; c0 += 32) {
    const int col = c0 + cb;
    const bool live = col < dv;
    float next[R];
    if (c0 + 32 < dv) load_column<R>(next, head + (size_t)(col + 32) * dk, dk, rg, pos > 0 && col + 32 < dv);
    float dot = 0.f, o = 0.f;
#pragma unroll
    for (int m = 0; m < R; ++m) {
      S[m] *= gg[m];
      dot = fmaf(S[m], kk[m], dot);
    }
    dot = sum8(dot);
    const float u = live ? beta * (vs[col] - dot) : 0.f;
#pragma unroll
    for (int m = 0; m < R; ++m) {
      S[m] = fmaf(kk[m], u, S[m]);
      o = fmaf(S[m], qq[m], o);
    }
    o = sum8(o);
    store_column<R>(S, head + (size_t)(live ? col : 0) * dk, dk, rg, live);
    if (rg == 0 && live) {
      os[col] = o;
      ss = fmaf(o, o, ss);
    }
    if (c0 + 32 < dv) {
#pragma unroll
      for (int m = 0; m < R; ++m) S[m] = next[m];
    }
  }
  ss = wave_sum(ss);
  if (lane == 0) parts[4 + wave] = ss;
  __syncthreads();
  const float s = 1.0f / sqrtf((parts[4] + parts[5] + parts[6] + parts[7]) / (float)dv + gt.eps);
  for (int c = tid; c < dv; c += 256)
    out[(size_t)t * ldo + (size_t)h * dv + c] = from_f<T>(gt.w[c] * (os[c] * s) * gt.template at<T>(t, h * dv + c));
}

// ------------------------------------------------------------------------------------------------ out
// Rows first .. first + n - 1: sixteen lanes a (row, head).
template <typename T>
__global__ __launch_bounds__(256) void out_kernel(const float* __restrict__ o, Gate gt, T* __restrict__ out, int ldo, int first, int n,
                                                  int H, int dv) {
  const long long pair = (long long)blockIdx.x * 16 + threadIdx.x / 16;
  const int li = threadIdx.x % 16;
  if (pair >= (long long)n * H) return;
  const int t = first + (int)(pair / H), h = (int)(pair % H);
  const float* orow = o + ((size_t)t * H + h) * dv;
  float ss = 0.f;
  for (int c = li; c < dv; c += 16) ss = fmaf(orow[c], orow[c], ss);
  const float s = 1.0f / sqrtf(sum16(ss) / (float)dv + gt.eps);
  for (int c = li; c < dv; c += 16)
    out[(size_t)t * ldo + (size_t)h * dv + c] = from_f<T>(gt.w[c] * (orow[c] * s) * gt.template at<T>(t, h * dv + c));
}

// The same in words of four channels (dv a multiple of 4 up to 256, aligned rows).
template <typename T>
__global__ __launch_bounds__(256) void out_words_kernel(const float* __restrict__ o, Gate gt, T* __restrict__ out, int ldo, int first,
                                                        int n, int H, int dv) {
  typedef T quad __attribute__((ext_vector_type(4)));
  const long long pair = (long long)blockIdx.x * 16 + threadIdx.x / 16;
  const int li = threadIdx.x % 16;
  if (pair >= (long long)n * H) return;
  const int t = first + (int)(pair / H), h = (int)(pair % H);
  const float* orow = o + ((size_t)t * H + h) * dv;
  f32x4 x[4];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = (i * 16 + li) * 4;
    if (c < dv) {
      x[i] = *reinterpret_cast<const f32x4*>(orow + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(x[i][e], x[i][e], ss);
    }
  }
  const float s = 1.0f / sqrtf(sum16(ss) / (float)dv + gt.eps);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = (i * 16 + li) * 4;
    if (c < dv) {
      f32x4 gv;
      if (gt.f32) {
        gv = *reinterpret_cast<const f32x4*>(static_cast<const float*>(gt.gate) + (size_t)t * gt.ld + h * dv + c);
      } else {
        const quad gq = *reinterpret_cast<const quad*>(static_cast<const T*>(gt.gate) + (size_t)t * gt.ld + h * dv + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) gv[e] = to_f(gq[e]);
      }
      const f32x4 w = *reinterpret_cast<const f32x4*>(gt.w + c);
      quad y;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float a = sigmoid(gv[e]);
        y[e] = from_f<T>(w[e] * (x[i][e] * s) * (gt.sigmoid ? a : gv[e] * a));
      }
      *reinterpret_cast<quad*>(out + (size_t)t * ldo + (size_t)h * dv + c) = y;
    }
  }
}

// ------------------------------------------------------------------------------------------------ chunks
// Where a (chunk, head)'s pieces lie in the workspace, in floats: Q' [64][dkp], O' turned [dvp][64], M [dkp][dkp], B turned
// [dvp][dkp], the state before the chunk as a slot holds it [dvp][dkp].  Chunks of a request follow one another from number
// (its first row - the portions' first row) / 64 + its number among the portions.
struct Pieces {
  int dkp, dvp;
  __host__ __device__ __forceinline__ long long q() const { return 0; }
  __host__ __device__ __forceinline__ long long o() const { return (long long)kC * dkp; }
  __host__ __device__ __forceinline__ long long m() const { return o() + (long long)kC * dvp; }
  __host__ __device__ __forceinline__ long long b() const { return m() + (long long)dkp * dkp; }
  __host__ __device__ __forceinline__ long long s() const { return b() + (long long)dvp * dkp; }
  __host__ __device__ __forceinline__ long long floats() const { return s() + (long long)dvp * dkp; }
};
__device__ __forceinline__ int chunk_base(const Rows& rw, int seq, int seq_base, int first_row) {
  return (rw.q_start[seq] - first_row) / kC + (seq - seq_base);
}

struct ChunkPlace {
  int h, seq, ci;
  bool ok;
  __device__ __forceinline__ ChunkPlace(int H, int seq_base, int units, int chunks) {
    const int within = blockIdx.x / 8, unit = within / H * 8 + blockIdx.x % 8;
    h = within % H;
    ok = unit < units;
    seq = seq_base + (ok ? unit / chunks : 0);
    ci = unit % chunks;
  }
};

__device__ __forceinline__ f32x4 mfma4(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

constexpr int kLA = kC + 4;   // row stride of what has a column a token
template <int DKP, bool CHANNEL>
constexpr int chunk_floats_of_lds() {
  const int rows = kC * (DKP + 4), turned = DKP * kLA;
  return (CHANNEL && DKP <= 64 ? rows : 0) + 2 * rows + (CHANNEL ? (rows > turned ? rows : turned) : kC + turned) + 2 * kC * kLA + 4 * 16 * 20 + kC + DKP;
}

// MFMA operands: lane (x = lane % 16, kq = lane / 16).  Over 16 of k in four instructions, instruction s takes k = 4 kq + s of both
// operands; a result lane then holds column x and rows 4 kq .. 4 kq + 3, which is as it stands the right operand of a product
// over those rows.
//
// A one-dimensional grid of 8 * heads * ceil(units / 8), eight waves each: a unit is a chunk of a request, `chunks` of them a request
// from seq_base on.  A die (see chain_kernel) takes all heads of a chunk: neighbouring columns of the same rows.
template <typename T, int DKP, bool CHANNEL>
__global__ __launch_bounds__(512) void chunk_kernel(const T* __restrict__ proj, Proj p, const float* __restrict__ wconv, Decay dc, Rows rw,
                                                    Sizes sz, int seq_base, int units, int chunks, int first_row, float q_scale, int words,
                                                    float* __restrict__ ws, Pieces pc) {
  constexpr int LD = DKP + 4, THREADS = 512, WAVES = 8, LPR = DKP / 4;
  extern __shared__ float lds[];
  float* Ks = lds;                    // [64][LD]: k, later e^G k
  float* Qs = Ks + kC * LD;           // [64][LD]: q, later e^G q
  float* Gs = Qs + kC * LD;           // CHANNEL: [64][LD], else [64]: the log decays (of 2), then their sums up to and with each token
  float* KT = CHANNEL ? Gs : Gs + kC;   // [DKP][kLA]: e^(G_last - G) k turned (with CHANNEL in the place of the sums)
  float* NA = CHANNEL ? Gs + (kC * LD > DKP * kLA ? kC * LD : DKP * kLA) : KT + DKP * kLA;   // [64][kLA]: -A
  float* Ps = NA + kC * kLA;          // [64][kLA]: P
  float* X = Ps + kC * kLA;           // [4][16][20]: the inverses of the diagonal blocks of I + A
  float* Bs = X + 4 * 16 * 20;        // [64]: beta
  float* Ge = Bs + kC;                // [DKP]: e^(G_last)
  constexpr bool OWN = CHANNEL && DKP <= 64;
  float* Ds = Ge + DKP;               // OWN: [64][LD]: the decays themselves (where LDS has room for them)
  const ChunkPlace place(sz.H, seq_base, units, chunks);
  const int seq = place.seq, ci = place.ci, h = place.h;
  const int L = rw.q_len[seq];
  if (!place.ok || ci * kC >= L) return;
  const int H = sz.H, G = sz.G, dk = sz.dk, dv = sz.dv, g = h / (H / G), taps = sz.taps, channels = 2 * G * dk + H * dv;
  const int count = min(kC, L - ci * kC), off0 = ci * kC, pos0 = rw.pos0[seq];
  const int row0 = rw.q_start[seq] + off0;
  const float* ring = rw.state + (size_t)rw.slots[seq] * rw.slot_floats + rw.ring_at;
  float* cell = ws + ((size_t)(chunk_base(rw, seq, seq_base, first_row) + ci) * H + h) * pc.floats();
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave, x = lane % 16, kq = lane / 16;

  // the operands of the recurrence: a row's lanes take four channels each, ROWS rows at a time
  {
    const int c = tid % LPR * 4, qch = g * dk + c, kch = (G + g) * dk + c, t_min = row0 - off0;
    f32x4 dt = {0.f, 0.f, 0.f, 0.f};
    const float rate2 = -kLog2e * dc.rate[h];   // (log decays in units of log2)
    if (CHANNEL) {
#pragma unroll
      for (int e = 0; e < 4; ++e) dt[e] = c + e < dk ? dc.dt[h * dk + c + e] : 0.f;
    }
    // rows whose inputs are not all the step's, and channels that are no whole words, one input after the other
    auto slowly = [&](int ch, int size, int i) {
      f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (e < size) v[e] = convolved(proj, p, wconv, taps, channels, ch + e, row0 + i, off0 + i, pos0 + off0 + i, ring);
      return v;
    };
    constexpr int ROWS = 2, STEP = THREADS / LPR;
    static_assert(kC % (ROWS * STEP) == 0, "whole rounds of rows");
    for (int i0 = tid / LPR; i0 < kC; i0 += ROWS * STEP) {
      f32x4 qv[ROWS], kv[ROWS], zv[ROWS];
      if (words) {
        const int cc = c < dk ? c : 0;
        auto rows = [&](auto mt) {
#pragma unroll
          for (int n = 0; n < ROWS; ++n) {
            const int t = row0 + min(i0 + n * STEP, count - 1);
            qv[n] = convolved4_rows<T, mt.value>(proj, p, wconv, taps, channels, g * dk + cc, t, t_min);
            kv[n] = convolved4_rows<T, mt.value>(proj, p, wconv, taps, channels, (G + g) * dk + cc, t, t_min);
          }
        };
        if (taps <= 4) rows(std::integral_constant<int, 4>{});
        else rows(std::integral_constant<int, kMaxTaps>{});
      }
      if (CHANNEL) {
#pragma unroll
        for (int n = 0; n < ROWS; ++n) {
          const float* zr = dc.z + (size_t)(row0 + min(i0 + n * STEP, count - 1)) * dc.ldz + h * dk;
#pragma unroll
          for (int e = 0; e < 4; ++e) zv[n][e] = zr[min(c + e, dk - 1)];
        }
      }
#pragma unroll
      for (int n = 0; n < ROWS; ++n) {
        const int i = i0 + n * STEP, size = i < count ? dk - c : 0;
        if (size > 0 && (!words || off0 + i < taps - 1)) {
          qv[n] = slowly(qch, size, i);
          kv[n] = slowly(kch, size, i);
        }
        float sq = 0.f, sk = 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float a = e < size ? silu(qv[n][e]) : 0.f, b = e < size ? silu(kv[n][e]) : 0.f;
          qv[n][e] = a;
          kv[n][e] = b;
          sq = fmaf(a, a, sq);
          sk = fmaf(b, b, sk);
        }
#pragma unroll
        for (int o = 1; o < LPR; o <<= 1) {
          sq += __shfl_xor(sq, o, kWave);
          sk += __shfl_xor(sk, o, kWave);
        }
        *reinterpret_cast<f32x4*>(Qs + i * LD + c) = qv[n] * (q_scale / sqrtf(sq + 1e-6f));
        *reinterpret_cast<f32x4*>(Ks + i * LD + c) = kv[n] * (1.0f / sqrtf(sk + 1e-6f));
        if (CHANNEL) {
          f32x4 lg;
#pragma unroll
          for (int e = 0; e < 4; ++e) lg[e] = e < size ? rate2 * softplus(zv[n][e] + dt[e]) : 0.f;
          *reinterpret_cast<f32x4*>(Gs + i * LD + c) = lg;
          if (OWN) *reinterpret_cast<f32x4*>(Ds + i * LD + c) = f32x4{exp2_of(lg[0]), exp2_of(lg[1]), exp2_of(lg[2]), exp2_of(lg[3])};
        }
      }
    }
    // the values, a lane a token: they wait turned, [dvp][64], where O' will be
    for (int cv = wave * 4; cv < pc.dvp; cv += WAVES * 4) {
      const int i = lane, ch = 2 * G * dk + h * dv + cv, size = i < count ? dv - cv : 0;
      f32x4 v = {0.f, 0.f, 0.f, 0.f};
      if (words && cv < dv) {
        const int t = row0 + min(i, count - 1);
        v = taps <= 4 ? convolved4_rows<T, 4>(proj, p, wconv, taps, channels, ch, t, t_min)
                      : convolved4_rows<T, kMaxTaps>(proj, p, wconv, taps, channels, ch, t, t_min);
      }
      if (size > 0 && (!words || off0 + i < taps - 1)) v = slowly(ch, size, i);
#pragma unroll
      for (int e = 0; e < 4; ++e) cell[pc.o() + (cv + e) * kC + i] = e < size ? to_f(from_f<T>(silu(v[e]))) : 0.f;
    }
    if (tid < kC) {
      const T* row = proj + (size_t)(row0 + min(tid, count - 1)) * p.ld;
      Bs[tid] = tid < count ? sigmoid(to_f(row[p.b_at + h])) : 0.f;
      if (!CHANNEL) Gs[tid] = tid < count ? rate2 * softplus(to_f(row[p.a_at + h]) + dc.dt[h]) : 0.f;
    }
  }
  __syncthreads();

  // the blocks of A and P, 16 x 16.  On the diagonal with a decay a channel: from the log decays before they are summed up
  if constexpr (CHANNEL) {
    // waves 2 b and 2 b + 1: diagonal block b, eight of its columns each.  Lane (jl = lane / 8, ce = lane % 8): token j of the
    // block and the words of four channels ce, ce + 8, ...; row i after row i, with the pair's decay as a running product
    constexpr int NW = DKP / 32;
    const int b0 = 16 * (wave / 2), j = 8 * (wave % 2) + lane / 8, ce = lane % 8;
    f32x4 kj[NW], E[NW];
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      kj[w] = *reinterpret_cast<const f32x4*>(Ks + (b0 + j) * LD + (w * 8 + ce) * 4);
      E[w] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll 4
    for (int i = 0; i < 16; ++i) {
      float a = 0.f, pq = 0.f;
      const bool start = i == j;
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        const int at = (b0 + i) * LD + (w * 8 + ce) * 4;
        const f32x4 ki = *reinterpret_cast<const f32x4*>(Ks + at), qi = *reinterpret_cast<const f32x4*>(Qs + at);
        f32x4 gi = *reinterpret_cast<const f32x4*>((OWN ? Ds : Gs) + at);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          if (!OWN) gi[e] = exp2_of(gi[e]);
          E[w][e] = start ? kj[w][e] : E[w][e] * gi[e];   // k_j times the decay from j to i (zero before j)
          a = fmaf(ki[e], E[w][e], a);
          pq = fmaf(qi[e], E[w][e], pq);
        }
      }
      a = sum8(a);
      pq = sum8(pq);
      if (ce == 0) {
        NA[(b0 + i) * kLA + b0 + j] = j < i ? -Bs[b0 + i] * a : 0.f;
        Ps[(b0 + i) * kLA + b0 + j] = pq;   // (zero for j > i)
      }
    }
    __syncthreads();
    if (tid < DKP) {   // the sums of the log decays, a thread a channel
      float sum = 0.f;
#pragma unroll 16
      for (int i = 0; i < kC; ++i) {
        sum += Gs[i * LD + tid];
        Gs[i * LD + tid] = sum;
      }
    }
  } else {
    if (wave == 0) {
      float sum = Gs[lane];
#pragma unroll
      for (int o = 1; o < kC; o <<= 1) {
        const float other = __shfl_up(sum, o, kWave);
        if (lane >= o) sum += other;
      }
      Gs[lane] = sum;
    }
  }
  __syncthreads();
  // blocks (I, J) below the diagonal (and on it without a decay a channel), dealt to the waves
  for (int blk = wave; blk < (CHANNEL ? 6 : 10); blk += WAVES) {
    int I, J;
    if (CHANNEL) I = blk < 1 ? 1 : blk < 3 ? 2 : 3, J = blk - I * (I - 1) / 2;
    else I = blk < 1 ? 0 : blk < 3 ? 1 : blk < 6 ? 2 : 3, J = blk - I * (I + 1) / 2;
    f32x4 a = {0.f, 0.f, 0.f, 0.f}, pq = a;
    const int iat = (16 * I + x) * LD, jat = (16 * J + x) * LD;
#pragma unroll
    for (int c0 = 0; c0 < DKP; c0 += 16) {
      const int c = c0 + 4 * kq;
      f32x4 ki = *reinterpret_cast<const f32x4*>(Ks + iat + c), qi = *reinterpret_cast<const f32x4*>(Qs + iat + c);
      f32x4 kj = *reinterpret_cast<const f32x4*>(Ks + jat + c);
      if constexpr (CHANNEL) {
        const f32x4 ref = *reinterpret_cast<const f32x4*>(Gs + (16 * I - 1) * LD + c);
        const f32x4 gi = *reinterpret_cast<const f32x4*>(Gs + iat + c), gj = *reinterpret_cast<const f32x4*>(Gs + jat + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float from = exp2_of(gi[e] - ref[e]);
          ki[e] *= from;
          qi[e] *= from;
          kj[e] *= exp2_of(ref[e] - gj[e]);
        }
      }
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        a = mfma4(ki[s], kj[s], a);
        pq = mfma4(qi[s], kj[s], pq);
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * I + 4 * kq + r, j = 16 * J + x;
      float d = 1.f;
      if (!CHANNEL) d = j <= i ? exp2_of(Gs[i] - Gs[j]) : 0.f;
      NA[i * kLA + j] = j < i ? -Bs[i] * a[r] * d : 0.f;
      Ps[i * kLA + j] = j <= i ? pq[r] * d : 0.f;
    }
  }
  __syncthreads();
  // waves 4 .. 7: the inverse of diagonal block w of I + A, lane j < 16 its column j
  if (wave >= 4 && lane < 16) {
    const int b = wave - 4;
    float col[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float sum = i == lane ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) sum = fmaf(NA[(16 * b + i) * kLA + 16 * b + m], col[m], sum);
      col[i] = sum;
      X[(b * 16 + i) * 20 + lane] = sum;
    }
  }
  {   // e^G on queries and keys, and the keys' decay to the chunk's end
    constexpr int PER = kC * DKP / THREADS;
    float turned[PER];
#pragma unroll
    for (int n = 0; n < PER; ++n) {
      const int idx = tid + n * THREADS, i = idx / DKP, c = idx % DKP;
      const float gi = CHANNEL ? Gs[i * LD + c] : Gs[i], last = CHANNEL ? Gs[(kC - 1) * LD + c] : Gs[kC - 1];
      const float kv = Ks[i * LD + c], e = exp2_of(gi);
      turned[n] = kv * exp2_of(last - gi);
      Ks[i * LD + c] = kv * e;
      Qs[i * LD + c] *= e;
      if (i == 0) Ge[c] = exp2_of(last);
    }
    __syncthreads();
#pragma unroll
    for (int n = 0; n < PER; ++n) {
      const int idx = tid + n * THREADS, i = idx / DKP, c = idx % DKP;
      KT[c * kLA + i] = turned[n];
    }
  }
  __syncthreads();
  // 16 columns of W or U at a time: block row after block row, (I + A) Y = right side; then P Y and the turned keys times Y
  const int tiles = DKP / 16 + pc.dvp / 16;
  for (int tile = wave; tile < tiles; tile += WAVES) {
    const bool is_w = tile < DKP / 16;
    const int c = (is_w ? tile : tile - DKP / 16) * 16 + x;
    f32x4 y[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      const int i0 = 16 * I + 4 * kq;
      f32x4 acc;
      if (is_w) {
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[r] = Ks[(i0 + r) * LD + c];
      } else {
        acc = *reinterpret_cast<const f32x4*>(cell + pc.o() + c * kC + i0);
      }
      acc *= *reinterpret_cast<const f32x4*>(Bs + i0);
#pragma unroll
      for (int J = 0; J < I; ++J) {
        const f32x4 na = *reinterpret_cast<const f32x4*>(NA + (16 * I + x) * kLA + 16 * J + 4 * kq);
#pragma unroll
        for (int s = 0; s < 4; ++s) acc = mfma4(na[s], y[J][s], acc);
      }
      const f32x4 xi = *reinterpret_cast<const f32x4*>(X + (I * 16 + x) * 20 + 4 * kq);
      f32x4 res = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 4; ++s) res = mfma4(xi[s], acc[s], res);
      y[I] = res;
    }
    f32x4 py[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) py[I] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int J = 0; J < 4; ++J)
#pragma unroll
      for (int I = J; I < 4; ++I) {
        const f32x4 pij = *reinterpret_cast<const f32x4*>(Ps + (16 * I + x) * kLA + 16 * J + 4 * kq);
#pragma unroll
        for (int s = 0; s < 4; ++s) py[I] = mfma4(pij[s], y[J][s], py[I]);
      }
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      if (is_w) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = 16 * I + 4 * kq + r;
          cell[pc.q() + i * DKP + c] = Qs[i * LD + c] - py[I][r];
        }
      } else {
        *reinterpret_cast<f32x4*>(cell + pc.o() + c * kC + 16 * I + 4 * kq) = py[I];
      }
    }
#pragma unroll 1   // (unrolled, the operands of all of them would want registers at once)
    for (int ct = 0; ct < DKP / 16; ct += 2) {
      f32x4 ky[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
      for (int J = 0; J < 4; ++J) {
        const f32x4 k0 = *reinterpret_cast<const f32x4*>(KT + (16 * ct + x) * kLA + 16 * J + 4 * kq);
        const f32x4 k1 = *reinterpret_cast<const f32x4*>(KT + (16 * ct + 16 + x) * kLA + 16 * J + 4 * kq);
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          ky[0] = mfma4(k0[s], y[J][s], ky[0]);
          ky[1] = mfma4(k1[s], y[J][s], ky[1]);
        }
      }
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const int r0 = 16 * (ct + t) + 4 * kq;
        if (is_w) {
#pragma unroll
          for (int r = 0; r < 4; ++r) cell[pc.m() + (r0 + r) * DKP + c] = (r0 + r == c ? Ge[c] : 0.f) - ky[t][r];
        } else {
          *reinterpret_cast<f32x4*>(cell + pc.b() + c * DKP + r0) = ky[t];
        }
      }
    }
  }
}

// The walk, S <- M S + B: four waves a workgroup, 16 columns of a (request, head); wave w holds a quarter of S's rows (DKP / 64 tiles
// of 16), S as a whole passes between the waves through LDS.  The operands of the next three chunks are on their way while a
// chunk is worked on.  A one-dimensional grid of 8 * columns * ceil(units / 8): the chip deals workgroups round its eight dies,
// and the workgroups of a (request, head), which read the same M, are put on one.
template <int DKP>
struct ChainOperands {
  static constexpr int KT = DKP / 16, ST = DKP / 64;
  f32x4 m[ST][KT], b[ST];
  __device__ __forceinline__ void fetch(const float* __restrict__ at, const Pieces& pc, int w, int x, int kq, int col) {
#pragma unroll
    for (int i = 0; i < ST; ++i) {
#pragma unroll
      for (int t = 0; t < KT; ++t) m[i][t] = *reinterpret_cast<const f32x4*>(at + pc.m() + ((w * ST + i) * 16 + x) * DKP + 16 * t + 4 * kq);
      b[i] = *reinterpret_cast<const f32x4*>(at + pc.b() + col * DKP + (w * ST + i) * 16 + 4 * kq);
    }
  }
};

template <int DKP>
__global__ __launch_bounds__(256, 1) void chain_kernel(Rows rw, Sizes sz, int seq_base, int units, int first_row, float* __restrict__ ws,
                                                    Pieces pc) {
  constexpr int KT = DKP / 16, ST = DKP / 64, LS = DKP + 4, AHEAD = 4;
  __shared__ float Ss[2][16 * LS];    // [column][channel], the state before and behind a chunk in turn
  const int cols = pc.dvp / 16, place = blockIdx.x / 8;
  const int unit = place / cols * 8 + blockIdx.x % 8;
  if (unit >= units) return;
  const int seq = seq_base + unit / sz.H, h = unit % sz.H, col0 = place % cols * 16;
  const int tid = threadIdx.x, lane = tid % kWave, w = tid / kWave, x = lane % 16, kq = lane / 16;
  const int H = sz.H, dk = sz.dk, dv = sz.dv, L = rw.q_len[seq], col = col0 + x;
  const bool live = col < dv, begun = rw.pos0[seq] > 0;
  float* column = rw.state + (size_t)rw.slots[seq] * rw.slot_floats + ((size_t)h * dv + (live ? col : 0)) * dk;
  const int chunks = (L + kC - 1) / kC;
  float* cell = ws + ((size_t)chunk_base(rw, seq, seq_base, first_row) * H + h) * pc.floats();
  const size_t cell_step = (size_t)H * pc.floats();

  ChainOperands<DKP> op[AHEAD];
#pragma unroll
  for (int a = 0; a < AHEAD - 1; ++a) op[a].fetch(cell + (size_t)min(a, chunks - 1) * cell_step, pc, w, x, kq, col);
  f32x4 S[ST];   // rows (w ST + i) 16 + 4 kq + r, column x
#pragma unroll
  for (int i = 0; i < ST; ++i) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int c = (w * ST + i) * 16 + 4 * kq + r;
      S[i][r] = begun && live && c < dk ? column[c] : 0.f;
    }
    *reinterpret_cast<f32x4*>(&Ss[0][x * LS + (w * ST + i) * 16 + 4 * kq]) = S[i];
  }
  auto work = [&](int ci, const ChainOperands<DKP>& at) {
#pragma unroll
    for (int i = 0; i < ST; ++i) *reinterpret_cast<f32x4*>(cell + (size_t)ci * cell_step + pc.s() + col * DKP + (w * ST + i) * 16 + 4 * kq) = S[i];
    __syncthreads();   // S is in LDS (and what the chunk before read has been read)
    f32x4 sb[KT];
#pragma unroll
    for (int t = 0; t < KT; ++t) sb[t] = *reinterpret_cast<const f32x4*>(&Ss[ci & 1][x * LS + 16 * t + 4 * kq]);
#pragma unroll
    for (int i = 0; i < ST; ++i) {
      f32x4 s0 = at.b[i], s1 = {0.f, 0.f, 0.f, 0.f};   // (two sums, so that neighbouring instructions do not wait for one another)
#pragma unroll
      for (int t = 0; t < KT; ++t)
#pragma unroll
        for (int s = 0; s < 4; s += 2) {
          s0 = mfma4(at.m[i][t][s], sb[t][s], s0);
          s1 = mfma4(at.m[i][t][s + 1], sb[t][s + 1], s1);
        }
      S[i] = s0 + s1;
      *reinterpret_cast<f32x4*>(&Ss[1 - (ci & 1)][x * LS + (w * ST + i) * 16 + 4 * kq]) = S[i];
    }
  };
  for (int ci = 0; ci < chunks; ci += AHEAD) {   // (chunks beyond the last one are read from the last one's place again)
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      if (ci + a >= chunks) break;
      op[(a + AHEAD - 1) % AHEAD].fetch(cell + (size_t)min(ci + a + AHEAD - 1, chunks - 1) * cell_step, pc, w, x, kq, col);
      __builtin_amdgcn_sched_barrier(0);
      work(ci + a, op[a]);
    }
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < ST; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = (w * ST + i) * 16 + 4 * kq + r;
        if (c < dk) column[c] = S[i][r];
      }
  }
}

// o = Q' S0 + O' of a (chunk, head), normed and gated: four waves of 16 tokens each, a token's dv columns in NT tiles of 16.
// The grid of chunk_kernel.
template <typename T, int DKP, int NT>
__global__ __launch_bounds__(256) void emit_kernel(Rows rw, Sizes sz, int seq_base, int units, int chunks, int first_row, const float* __restrict__ ws, Pieces pc,
                                                   Gate gt, T* __restrict__ out, int ldo) {
  constexpr int KT = DKP / 16;
  const ChunkPlace place(sz.H, seq_base, units, chunks);
  const int seq = place.seq, ci = place.ci, h = place.h;
  const int L = rw.q_len[seq];
  if (!place.ok || ci * kC >= L) return;
  const int H = sz.H, dv = sz.dv, tid = threadIdx.x, lane = tid % kWave, w = tid / kWave, x = lane % 16, kq = lane / 16;
  const int count = min(kC, L - ci * kC), tiles = pc.dvp / 16;
  const size_t row0 = (size_t)rw.q_start[seq] + (size_t)ci * kC;
  const float* cell = ws + ((size_t)(chunk_base(rw, seq, seq_base, first_row) + ci) * H + h) * pc.floats();
  f32x4 qf[KT], o[NT];
#pragma unroll
  for (int t = 0; t < KT; ++t) qf[t] = *reinterpret_cast<const f32x4*>(cell + pc.q() + (16 * w + x) * DKP + 16 * t + 4 * kq);
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    o[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (n < tiles) o[n] = *reinterpret_cast<const f32x4*>(cell + pc.o() + (16 * n + x) * kC + 16 * w + 4 * kq);
  }
  float ss[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    if (n < tiles) {
      f32x4 o1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int t = 0; t < KT; ++t) {
        const f32x4 sb = *reinterpret_cast<const f32x4*>(cell + pc.s() + (16 * n + x) * DKP + 16 * t + 4 * kq);
#pragma unroll
        for (int s = 0; s < 4; s += 2) {
          o[n] = mfma4(qf[t][s], sb[s], o[n]);
          o1 = mfma4(qf[t][s + 1], sb[s + 1], o1);
        }
      }
      o[n] += o1;   // (columns beyond dv are zero)
#pragma unroll
      for (int r = 0; r < 4; ++r) ss[r] = fmaf(o[n][r], o[n][r], ss[r]);
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) ss[r] = 1.0f / sqrtf(sum16(ss[r]) / (float)dv + gt.eps);
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int c = 16 * n + x;
    const float wn = c < dv ? gt.w[c] : 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * w + 4 * kq + r;
      if (i < count && c < dv)
        out[(row0 + i) * ldo + (size_t)h * dv + c] = from_f<T>(wn * (o[n][r] * ss[r]) * gt.template at<T>(row0 + i, h * dv + c));
    }
  }
}

inline bool words16(const void* p) { return (uintptr_t)p % 16 == 0; }

int check(const Sizes& sz, const Rows& rw, const char* what) {
  GB_REQUIRE(sz.H > 0 && sz.G > 0 && sz.H % sz.G == 0 && sz.dk > 0 && sz.dv > 0, "%s: bad heads H=%d G=%d dk=%d dv=%d", what, sz.H, sz.G, sz.dk, sz.dv);
  GB_REQUIRE(sz.dk <= 256, "%s: a key size of %d is above the supported 256", what, sz.dk);
  GB_REQUIRE(sz.taps >= 1 && sz.taps <= kMaxTaps, "%s: %d taps (1 to %d)", what, sz.taps, kMaxTaps);
  const long long S = (long long)sz.H * sz.dv * sz.dk, ring = sz.taps > 1 ? (long long)sz.taps * (2 * sz.G * sz.dk + sz.H * sz.dv) : 0;
  GB_REQUIRE(rw.ring_at >= S && rw.slot_floats >= rw.ring_at + ring && rw.ring_at % 4 == 0 && rw.slot_floats % 4 == 0 && words16(rw.state),
             "%s: a slot of %lld floats (the ring from %lld on) does not hold the state", what, rw.slot_floats, rw.ring_at);
  GB_REQUIRE(rw.tok_seq && rw.q_start && rw.q_len && rw.pos0 && rw.slots && rw.state, "%s: the step's tables and the state are needed", what);
  return 0;
}
int check_proj(const Sizes& sz, const Proj& p, const Decay& dc, const char* what) {
  const int channels = 2 * sz.G * sz.dk + sz.H * sz.dv;
  GB_REQUIRE(p.at >= 0 && p.at + channels <= p.ld && p.b_at >= 0 && p.b_at + sz.H <= p.ld, "%s: rows of %d are shorter than the projections", what, p.ld);
  GB_REQUIRE(dc.rate && dc.dt && (dc.channel ? dc.z && dc.ldz >= sz.H * sz.dk : p.a_at >= 0 && p.a_at + sz.H <= p.ld), "%s: the decay's logits are missing", what);
  return 0;
}
int move_ring(const void* proj, int dtype, const Proj& p, const Rows& rw, const Sizes& sz, int seq_base, int n_seqs, hipStream_t stream) {
  const int channels = 2 * sz.G * sz.dk + sz.H * sz.dv;
  const dim3 grid((unsigned)n_seqs, (unsigned)((channels + 255) / 256));
  if (dtype == kF32) hipLaunchKernelGGL(ring_kernel<float>, grid, dim3(256), 0, stream, (const float*)proj, p, rw, sz.taps, channels, seq_base);
  else hipLaunchKernelGGL(ring_kernel<bf16>, grid, dim3(256), 0, stream, (const bf16*)proj, p, rw, sz.taps, channels, seq_base);
  return launched("delta (ring)");
}
// whole words of four for the projections' channels
bool by_words(const Sizes& sz, const Proj& p, const void* proj, int dtype, const float* wconv) {
  const int bytes = dtype == kF32 ? 16 : 8;
  return sz.dk % 4 == 0 && sz.dv % 4 == 0 && p.at % 4 == 0 && p.ld % 4 == 0 && (uintptr_t)proj % bytes == 0 && words16(wconv);
}

}  // namespace

// proj [n, ld] of `dtype`; wconv float32 [taps, 2 G dk + H dv]; state float32 [slots, slot_floats].  Rows first .. first + n - 1 of
// the step, requests seq_base .. seq_base + n_seqs - 1; z float32 [n, ldz] (a decay a key channel) or nullptr (a decay a head, its
// logits at column a_at of proj); dv_taps = 16 dv + taps; q32, k32, v, beta, lg (see prep_kernel) are indexed by the step's row.
// The ring is moved on by a second kernel.  beta_lg: (first + n) H floats, filled up to a multiple of 4, then the log decays.
extern "C" int gb_delta_prep(const void* proj, int dtype, int ld, int at, int b_at, int a_at, const float* wconv, const float* rate,
                             const float* dt, const float* z, int ldz, const int32_t* tok_seq, const int32_t* q_start,
                             const int32_t* q_len, const int32_t* pos0, const int32_t* slots, float* state, long long slot_floats,
                             long long ring_at, int first, int n, int seq_base, int n_seqs, int H, int G, int dk, int dv_taps,
                             float* q32, float* k32, void* v, void* beta_lg, hipStream_t stream) {
  const int dv = dv_taps >> 4, taps = dv_taps & 15;
  const Rows rw{tok_seq, q_start, q_len, pos0, slots, state, slot_floats, ring_at};
  const Sizes sz{H, G, dk, dv, taps};
  const Proj p{ld, at, b_at, a_at};
  const int channel = z != nullptr;
  const Decay dc{rate, dt, z, ldz, channel};
  if (int rc = check(sz, rw, "delta_prep")) return rc;
  if (int rc = check_proj(sz, p, dc, "delta_prep")) return rc;
  GB_REQUIRE(n >= 0 && first >= 0 && n_seqs >= 0 && n_seqs <= 0x7fffffff && wconv && q32 && k32 && v && beta_lg, "delta_prep: bad arguments");
  if (n == 0 || n_seqs == 0) return 0;
  // beta [rows, H] comes first, the log decays behind it: rows = first + n of them
  float* beta = (float*)beta_lg;
  float* lg = beta + (((size_t)(first + n) * H + 3) & ~(size_t)3);
  const int units = 2 * G + H + (channel ? H : 1);
  const long long groups = (long long)n * units;
  GB_REQUIRE((groups + 15) / 16 < (1ll << 31), "delta_prep: too many (row, head) pairs");
  const dim3 grid((unsigned)((groups + 15) / 16));
  const float q_scale = 1.0f / sqrtf((float)dk);
  const bool w = by_words(sz, p, proj, dtype, wconv) && words16(q32) && words16(k32) && words16(v);
#define GB_PREP(T, W) hipLaunchKernelGGL((prep_kernel<T, W>), grid, dim3(256), 0, stream, (const T*)proj, p, wconv, dc, rw, sz, first, n, q32, k32, (T*)v, beta, lg, units, q_scale)
  if (dtype == kF32) {
    if (w) GB_PREP(float, true);
    else GB_PREP(float, false);
  } else if (dtype == kBF16) {
    if (w) GB_PREP(bf16, true);
    else GB_PREP(bf16, false);
  } else {
    return fail("delta_prep: unknown dtype %d", dtype);
  }
#undef GB_PREP
  if (int rc = launched("delta_prep")) return rc;
  return taps > 1 ? move_ring(proj, dtype, p, rw, sz, seq_base, n_seqs, stream) : 0;
}

// The recurrence token after token over requests seq_base .. of the step, whose rows are first .. first + n - 1: o [.., H dv] float32
// by the step's row.
extern "C" int gb_delta_scan(const float* q32, const float* k32, const void* v, int dtype, const void* beta_lg, int channel, float* out,
                             const int32_t* q_start, const int32_t* q_len, const int32_t* pos0, const int32_t* slots, float* state,
                             long long slot_floats, long long ring_at, int first, int n, int seq_base, int n_seqs, int H, int G, int dk,
                             int dv, hipStream_t stream) {
  const Rows rw{q_start, q_start, q_len, pos0, slots, state, slot_floats, ring_at};
  const Sizes sz{H, G, dk, dv, 1};
  if (int rc = check(sz, rw, "delta_scan")) return rc;
  GB_REQUIRE(n >= 0 && first >= 0 && n_seqs >= 0 && q32 && k32 && v && beta_lg && out && (dtype == kF32 || dtype == kBF16), "delta_scan: bad arguments");
  GB_REQUIRE(n_seqs <= 65535 && H <= 65535, "delta_scan: too many requests or heads for one launch");
  if (n == 0 || n_seqs == 0) return 0;
  const float* beta = (const float*)beta_lg;
  const float* lg = beta + (((size_t)(first + n) * H + 3) & ~(size_t)3);
  const dim3 grid((unsigned)((dv + 31) / 32), (unsigned)H, (unsigned)n_seqs);
  int R = 4;
  while (R * kLanesCol < dk) R *= 2;
#define GB_SCAN(RR)                                                                                                              \
  if (R == RR) {                                                                                                                 \
    if (dtype == kF32) hipLaunchKernelGGL((scan_kernel<float, RR>), grid, dim3(256), 0, stream, q32, k32, (const float*)v, beta, lg, channel, out, rw, sz, seq_base); \
    else hipLaunchKernelGGL((scan_kernel<bf16, RR>), grid, dim3(256), 0, stream, q32, k32, (const bf16*)v, beta, lg, channel, out, rw, sz, seq_base); \
  }
  GB_SCAN(4) GB_SCAN(8) GB_SCAN(16) GB_SCAN(32)
#undef GB_SCAN
  return launched("delta_scan");
}

// Floats of workspace for portions of `rows` rows in all in chunks, or 0 where these sizes go token by token.
extern "C" long long gb_delta_chunk_floats(int rows, int n_seqs, int H, int dk, int dv) {
  if (dk > 128 || dv > 256 || rows <= 0 || n_seqs <= 0) return 0;
  const Pieces pc{dk <= 64 ? 64 : 128, (dv + 15) / 16 * 16};
  return ((long long)rows / kC + n_seqs) * H * pc.floats();
}

// Portions in chunks, from the projections to the gated heads (arguments as gb_delta_prep and gb_delta_step take them; max_len: the
// longest portion's rows).  ws: workspace of gb_delta_chunk_floats floats.
extern "C" int gb_delta_chunks(const void* proj, int dtype, int ld, int at, int b_at, int a_at, const float* wconv, const float* rate,
                               const float* dt, const float* z, int ldz, const int32_t* q_start, const int32_t* q_len,
                               const int32_t* pos0, const int32_t* slots, float* state, long long slot_floats, long long ring_at,
                               int first, int n, int seq_base, int n_seqs, int max_len, int H, int G, int dk, int dv_taps,
                               const void* gate, int ldg, int gate_flags, const float* w, float eps, void* out, int ldo, float* ws,
                               long long ws_floats, hipStream_t stream) {
  const int dv = dv_taps >> 4, taps = dv_taps & 15, channel = z != nullptr;
  const Rows rw{q_start, q_start, q_len, pos0, slots, state, slot_floats, ring_at};
  const Sizes sz{H, G, dk, dv, taps};
  const Proj p{ld, at, b_at, a_at};
  const Decay dc{rate, dt, z, ldz, channel};
  if (int rc = check(sz, rw, "delta_chunks")) return rc;
  if (int rc = check_proj(sz, p, dc, "delta_chunks")) return rc;
  GB_REQUIRE(n >= 0 && first >= 0 && n_seqs >= 0 && wconv && gate && w && out && ws && ldg >= H * dv && ldo >= H * dv && (dtype == kF32 || dtype == kBF16),
             "delta_chunks: bad arguments");
  if (n == 0 || n_seqs == 0) return 0;
  GB_REQUIRE(dk <= 128 && dv <= 256 && max_len > 0 && ws_floats >= gb_delta_chunk_floats(n, n_seqs, H, dk, dv) && words16(ws),
             "delta_chunks: chunks need key sizes up to 128, value sizes up to 256 and a workspace of %lld floats", gb_delta_chunk_floats(n, n_seqs, H, dk, dv));
  const int chunks = (max_len + kC - 1) / kC;
  GB_REQUIRE((long long)n_seqs * H < (1ll << 20) && (long long)n_seqs * chunks * H < (1ll << 30), "delta_chunks: too many chunks, requests or heads for one launch");
  const Pieces pc{dk <= 64 ? 64 : 128, (dv + 15) / 16 * 16};
  const int units = n_seqs * H, words = by_words(sz, p, proj, dtype, wconv);
  const float q_scale = 1.0f / sqrtf((float)dk);
  const Gate gt{gate, ldg, gate_flags & 1, gate_flags >> 1 & 1, w, eps};
  const int chunk_units = n_seqs * chunks;
  const dim3 cgrid((unsigned)((chunk_units + 7) / 8 * 8 * H)), wgrid((unsigned)((units + 7) / 8 * 8 * (pc.dvp / 16)));
#define GB_CHUNK(T, D, CH)                                                                                                       \
  do {                                                                                                                           \
    const int lds = (int)sizeof(float) * chunk_floats_of_lds<D, CH>();                                                            \
    static bool set = false;                                                                                                     \
    if (!set) {                                                                                                                  \
      const hipError_t e = hipFuncSetAttribute((const void*)chunk_kernel<T, D, CH>, hipFuncAttributeMaxDynamicSharedMemorySize, lds); \
      if (e != hipSuccess) return fail("delta_chunks: %d bytes of LDS: %s", lds, hipGetErrorString(e));                           \
      set = true;                                                                                                                \
    }                                                                                                                            \
    hipLaunchKernelGGL((chunk_kernel<T, D, CH>), cgrid, dim3(512), lds, stream, (const T*)proj, p, wconv, dc, rw, sz, seq_base, chunk_units, chunks, first, \
                       q_scale, words, ws, pc);                                                                                  \
  } while (0)
#define GB_CHUNKS(T)                        \
  if (pc.dkp == 64) {                       \
    if (channel) GB_CHUNK(T, 64, true);     \
    else GB_CHUNK(T, 64, false);            \
  } else {                                  \
    if (channel) GB_CHUNK(T, 128, true);    \
    else GB_CHUNK(T, 128, false);           \
  }
  if (dtype == kF32) {
    GB_CHUNKS(float)
  } else {
    GB_CHUNKS(bf16)
  }
#undef GB_CHUNKS
#undef GB_CHUNK
  if (int rc = launched("delta_chunks")) return rc;
  if (taps > 1) {   // (the chunks have read what came before)
    if (int rc = move_ring(proj, dtype, p, rw, sz, seq_base, n_seqs, stream)) return rc;
  }
  if (pc.dkp == 64) hipLaunchKernelGGL(chain_kernel<64>, wgrid, dim3(256), 0, stream, rw, sz, seq_base, units, first, ws, pc);
  else hipLaunchKernelGGL(chain_kernel<128>, wgrid, dim3(256), 0, stream, rw, sz, seq_base, units, first, ws, pc);
  if (int rc = launched("delta_chunks (chain)")) return rc;
#define GB_EMIT(T, D, N) hipLaunchKernelGGL((emit_kernel<T, D, N>), cgrid, dim3(256), 0, stream, rw, sz, seq_base, chunk_units, chunks, first, (const float*)ws, pc, gt, (T*)out, ldo)
#define GB_EMITS(T, D)                         \
  do {                                         \
    if (pc.dvp <= 64) GB_EMIT(T, D, 4);        \
    else if (pc.dvp <= 128) GB_EMIT(T, D, 8);  \
    else GB_EMIT(T, D, 16);                    \
  } while (0)
  if (dtype == kF32) {
    if (pc.dkp == 64) GB_EMITS(float, 64);
    else GB_EMITS(float, 128);
  } else {
    if (pc.dkp == 64) GB_EMITS(bf16, 64);
    else GB_EMITS(bf16, 128);
  }
#undef GB_EMITS
#undef GB_EMIT
  return launched("delta_chunks (emit)");
}

// out[t, h, :] = w * o / sqrt(mean(o^2) + eps) * act(gate), rows first .. first + n - 1; gate [.., ldg] float32 (gate_f32) or of `dtype`.
extern "C" int gb_delta_out(const float* o, const void* gate, int ldg, int gate_f32, int sigmoid_gate, const float* w, float eps, void* out,
                            int dtype, int ldo, int first, int n, int H, int dv, hipStream_t stream) {
  GB_REQUIRE(n >= 0 && first >= 0 && H > 0 && dv > 0 && ldg >= H * dv && ldo >= H * dv && o && gate && w && out, "delta_out: bad sizes n=%d heads=%d dv=%d", n, H, dv);
  GB_REQUIRE(dtype == kF32 || dtype == kBF16, "delta_out: unknown dtype %d", dtype);
  if (n == 0) return 0;
  const Gate gt{gate, ldg, gate_f32, sigmoid_gate, w, eps};
  const long long pairs = (long long)n * H;
  GB_REQUIRE((pairs + 15) / 16 < (1ll << 31), "delta_out: too many (row, head) pairs");
  const dim3 grid((unsigned)((pairs + 15) / 16));
  const int gb = gate_f32 || dtype == kF32 ? 16 : 8, ob = dtype == kF32 ? 16 : 8;
  if (dv % 4 == 0 && dv <= 256 && ldg % 4 == 0 && ldo % 4 == 0 && words16(o) && words16(w) && (uintptr_t)gate % gb == 0 && (uintptr_t)out % ob == 0) {
    if (dtype == kF32) hipLaunchKernelGGL(out_words_kernel<float>, grid, dim3(256), 0, stream, o, gt, (float*)out, ldo, first, n, H, dv);
    else hipLaunchKernelGGL(out_words_kernel<bf16>, grid, dim3(256), 0, stream, o, gt, (bf16*)out, ldo, first, n, H, dv);
    return launched("delta_out");
  }
  if (dtype == kF32) hipLaunchKernelGGL(out_kernel<float>, grid, dim3(256), 0, stream, o, gt, (float*)out, ldo, first, n, H, dv);
  else hipLaunchKernelGGL(out_kernel<bf16>, grid, dim3(256), 0, stream, o, gt, (bf16*)out, ldo, first, n, H, dv);
  return launched("delta_out");
}

// Rows 0 .. n - 1, each the one row of request number t: from the projections to the gated heads.
extern "C" int gb_delta_step(const void* proj, int dtype, int ld, int at, int b_at, int a_at, const float* wconv, const float* rate,
                             const float* dt, const float* z, int ldz, const int32_t* q_start, const int32_t* pos0,
                             const int32_t* slots, float* state, long long slot_floats, long long ring_at, int n, int H, int G, int dk,
                             int dv_taps, const void* gate, int ldg, int gate_flags, const float* w, float eps, void* out, int ldo,
                             hipStream_t stream) {
  const int dv = dv_taps >> 4, taps = dv_taps & 15;
  const Rows rw{q_start, q_start, q_start, pos0, slots, state, slot_floats, ring_at};   // (row t is request t's only one)
  const Sizes sz{H, G, dk, dv, taps};
  const Proj p{ld, at, b_at, a_at};
  const int channel = z != nullptr;
  const Decay dc{rate, dt, z, ldz, channel};
  if (int rc = check(sz, rw, "delta_step")) return rc;
  if (int rc = check_proj(sz, p, dc, "delta_step")) return rc;
  GB_REQUIRE(n >= 0 && n <= 65535 && wconv && gate && w && out && ldg >= H * dv && ldo >= H * dv, "delta_step: bad arguments");
  GB_REQUIRE(dv <= 4096, "delta_step: a value size of %d is above the supported 4096", dv);
  if (n == 0) return 0;
  const Gate gt{gate, ldg, gate_flags & 1, gate_flags >> 1 & 1, w, eps};
  int R = 4;
  while (R * kLanesCol < dk) R *= 2;
  const size_t lds = sizeof(float) * (3 * (size_t)R * kLanesCol + 2 * (size_t)dv + 8);
  const float q_scale = 1.0f / sqrtf((float)dk);
  const dim3 grid((unsigned)H, (unsigned)n);
#define GB_STEP(RR)                                                                                                                    \
  if (R == RR) {                                                                                                                       \
    if (dtype == kF32) hipLaunchKernelGGL((step_kernel<float, RR>), grid, dim3(256), lds, stream, (const float*)proj, p, wconv, dc, rw, sz, q_scale, gt, (float*)out, ldo); \
    else if (dtype == kBF16) hipLaunchKernelGGL((step_kernel<bf16, RR>), grid, dim3(256), lds, stream, (const bf16*)proj, p, wconv, dc, rw, sz, q_scale, gt, (bf16*)out, ldo); \
    else return fail("delta_step: unknown dtype %d", dtype);                                                                           \
  }
  GB_STEP(4) GB_STEP(8) GB_STEP(16) GB_STEP(32)
#undef GB_STEP
  return launched("delta_step");
}

GB_TAPED(gb_delta_prep)
GB_TAPED(gb_delta_scan)
GB_TAPED(gb_delta_chunks)
GB_TAPED(gb_delta_out)
GB_TAPED(gb_delta_step)
