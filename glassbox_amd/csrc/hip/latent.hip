// Attention whose cache holds one latent row c of R channels a token instead of every head's key and value.  A head's key
// is W_uk c and its value W_uv c, so
//   score = q . (W_uk c) = (W_uk^T q) . c          and          sum_j p_j W_uv c_j = W_uv (sum_j p_j c_j) :
// a token that is decoded alone takes its queries into the latents' space, attends to the latents themselves (each is read
// once for all heads), and takes the sums through W_uv.  The tokens of a prompt portion, of which there are many for each
// key, get the keys and values of their request's whole context expanded into scratch pages instead, and go through the
// ordinary attention kernels.
//
//   latent_store    the RMS norm of a latent row and its way into the pages: [page][R / 8][slot][8] as a key head of R columns
//   latent_absorb   q' [n, H * R] = W_uk^T q, head by head; latent_store_absorb both in one launch
//   latent_decode   partial softmax sums of q' over a chunk of the context's latents, one workgroup a (chunk, 16 or 32 heads,
//                   token); latent_decode_plain the same for any sizes and types, a workgroup a (chunk, token, head)
//   latent_finish   the chunks' partial results added in their order, with the head's sink; W_uv; the sigmoid gate
//   latent_tables   the pages that the portions of a step expand into: one scratch page for each page of their contexts
//   latent_gather   the latents of those contexts as rows, zeros behind a context's end
//   latent_expand   rows [key heads | value heads] into the scratch pages (keys in pieces, values transposed)
//
// Scores and softmax are 32-bit and in units of log2: a weight is 2^(score * log2(e) - max).
#include "common.h"

using namespace gb;

GB_DEFINE_LAST_ERROR

namespace {

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kMaxRank = 2048;      // latents that the plain kernel and the last pass keep in LDS
constexpr int kMaxSplits = 256;     // chunks of a context that the last pass adds

__device__ __forceinline__ bf16x8 load8(const bf16* p) { return *reinterpret_cast<const bf16x8*>(p); }
__device__ __forceinline__ bf16x8 load8_once(const bf16* p) { return __builtin_nontemporal_load(reinterpret_cast<const bf16x8*>(p)); }
__device__ __forceinline__ bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int i = 0; i < 8; ++i) z[i] = (bf16)0.f;
  return z;
}
inline bool words16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }
inline bool grid_fits(long long count, int per_block) { return (count + per_block - 1) / per_block < (1ll << 31); }

// ------------------------------------------------------------------------------------------------ latent_store
// A wave a row.
template <typename T>
__device__ __forceinline__ void store_latent(const T* __restrict__ row, const float* __restrict__ gamma, float eps, int slot,
                                             T* __restrict__ pages, int page_size, int R, bool words, int lane) {
  T* page = pages + (size_t)(slot / page_size) * page_size * R;
  const int at = slot % page_size;
  float ss = 0.f;
  if constexpr (std::is_same<T, bf16>::value) {
    if (words) {   // rows of whole 16-byte words: a word is a piece
      for (int p = lane; p < R / 8; p += kWave) {
        const bf16x8 v = load8(row + 8 * p);
#pragma unroll
        for (int e = 0; e < 8; ++e) ss = fmaf((float)v[e], (float)v[e], ss);
      }
      ss = wave_sum(ss);
      const float r = 1.0f / sqrtf(ss / (float)R + eps);
      for (int p = lane; p < R / 8; p += kWave) {
        bf16x8 v = load8(row + 8 * p);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = (bf16)((float)v[e] * r * gamma[8 * p + e]);
        *reinterpret_cast<bf16x8*>(page + ((size_t)p * page_size + at) * 8) = v;
      }
      return;
    }
  }
  for (int c = lane; c < R; c += kWave) ss = fmaf(to_f(row[c]), to_f(row[c]), ss);
  ss = wave_sum(ss);
  const float r = 1.0f / sqrtf(ss / (float)R + eps);
  const int piece = key_piece(R);
  for (int c = lane; c < R; c += kWave) page[key_offset(at, c, page_size, piece)] = from_f<T>(to_f(row[c]) * r * gamma[c]);
}

template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(const T* __restrict__ in, int ld, const float* __restrict__ gamma, float eps,
                                                           const int32_t* __restrict__ slots, T* __restrict__ pages, int page_size,
                                                           int n, int R, int words) {
  const int t = blockIdx.x * 4 + threadIdx.x / kWave;
  if (t < n) store_latent(in + (size_t)t * ld, gamma, eps, slots[t], pages, page_size, R, words != 0, threadIdx.x % kWave);
}

// ------------------------------------------------------------------------------------------------ latent_absorb
// A wave a (64 latent channels, head, 16 tokens): D[channel][token], A = rows of W_uk^T ([H][R][hc], 16 bytes a lane), B =
// the tokens' queries.
__device__ __forceinline__ void absorb_tile(const bf16* __restrict__ q, int ldq, const bf16* __restrict__ uk_t, int hc,
                                            bf16* __restrict__ out, int n, int H, int R, int h, int r0, int t0, int lane) {
  const int j = lane & 15, c = lane >> 4;
  const int tok = t0 + j;
  f32x4 acc[4];
#pragma unroll
  for (int b = 0; b < 4; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < hc; k += 32) {
    const int k0 = k + 8 * c;
    const bf16x8 qf = (tok < n && k0 < hc) ? load8(q + (size_t)tok * ldq + (size_t)h * hc + k0) : zero8();
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const int r = r0 + 16 * b + j;
      const bf16x8 wf = (r < R && k0 < hc) ? load8(uk_t + ((size_t)h * R + r) * hc + k0) : zero8();
      acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, qf, acc[b], 0, 0, 0);
    }
  }
  if (tok >= n) return;
#pragma unroll
  for (int b = 0; b < 4; ++b) {
    const int r = r0 + 16 * b + 4 * c;
    if (r >= R) continue;   // (R is a multiple of 8)
    bf16x4 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = (bf16)acc[b][e];
    *reinterpret_cast<bf16x4*>(out + ((size_t)tok * H + h) * R + r) = o;
  }
}

__global__ __launch_bounds__(64) void latent_absorb_kernel(const bf16* __restrict__ q, int ldq, const bf16* __restrict__ uk_t, int hc,
                                                           bf16* __restrict__ out, int n, int H, int R) {
  absorb_tile(q, ldq, uk_t, hc, out, n, H, R, blockIdx.y, blockIdx.x * 64, blockIdx.z * 16, threadIdx.x);
}

// Both in one launch, for steps of few rows: workgroup y = H takes the latents (x counts rows), the others their tile of W_uk^T q
// for the first n_q tokens.
__global__ __launch_bounds__(64) void latent_store_absorb_kernel(const bf16* __restrict__ rows, int ld, int c_col, const float* __restrict__ gamma,
                                                                 float eps, const int32_t* __restrict__ slots, bf16* __restrict__ pages,
                                                                 int page_size, int n, const bf16* __restrict__ uk_t, int hc,
                                                                 bf16* __restrict__ out, int n_q, int H, int R) {
  if ((int)blockIdx.y == H) {
    for (int t = blockIdx.x + gridDim.x * blockIdx.z; t < n; t += gridDim.x * gridDim.z)
      store_latent(rows + (size_t)t * ld + c_col, gamma, eps, slots[t], pages, page_size, R, true, threadIdx.x);
    return;
  }
  absorb_tile(rows, ld, uk_t, hc, out, n_q, H, R, blockIdx.y, blockIdx.x * 64, blockIdx.z * 16, threadIdx.x);
}

// A thread a (token, head, channel): uk [H * hc, R], the first dim rows of a head.
template <typename T>
__global__ void latent_absorb_plain_kernel(const T* __restrict__ q, int ldq, const T* __restrict__ uk, int hc, int dim, T* __restrict__ out,
                                           long long count, int H, int R) {
  const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= count) return;
  const int r = (int)(idx % R), h = (int)(idx / R % H);
  const long long t = idx / R / H;
  const T* qr = q + (size_t)t * ldq + (size_t)h * hc;
  const T* w = uk + (size_t)h * hc * R + r;
  float acc = 0.f;
  for (int d = 0; d < dim; ++d) acc = fmaf(to_f(qr[d]), to_f(w[(size_t)d * R]), acc);
  out[idx] = from_f<T>(acc);
}

// ------------------------------------------------------------------------------------------------ latent_decode
// Four waves; a step takes 128 latents of the context.  Each wave reads 32 of them from their pages straight into MFMA
// operands (lane (j, c): key j, channels 32 ks + 8 c .. + 7, as the pages' pieces lie), forms the scores of its keys for all
// columns (a column is a head), and leaves scores and latents in LDS.  Then every wave takes part of the sums: per 32 keys it
// reads 8 keys x 8 channels a lane and turns them in registers (a pair of words gives two channels' pairs of keys), which makes
// eight operands of 16 channels, one of each run of eight; a column's running maximum is formed by each wave for itself, from
// the same scores in the same order.  The latents of the next step are on their way meanwhile.
//   S^T[key, col]     A = 16 keys x 32 channels,       B = 32 channels x 16 columns (the queries, in registers)
//   O^T[chan, col]    A = 16 channels x 32 keys,       B = 32 keys x 16 columns (the weights, as the lanes form them)
// KS: k-steps of 32 channels that hold R (FULL: exactly); CT: tiles of 16 columns.  The sums fall into units of (128 channels, tile of columns);
// with more waves than units the waves of a unit take its runs of 32 keys in turn, and their sums meet in LDS at the end.
template <int KS, int CT, bool FULL>
__global__ __launch_bounds__(256, 1) void latent_decode_kernel(const bf16* __restrict__ q, const bf16* __restrict__ pages,
                                                               const int32_t* __restrict__ tables, int table_stride,
                                                               const int32_t* __restrict__ positions, int H, int R, int P, float scale2,
                                                               int chunk, int splits, float* __restrict__ ws_acc,
                                                               float* __restrict__ ws_ml) {
  constexpr int KEYS = 128, KT = 2;         // keys a step; tiles of 16 of them a wave
  constexpr int ROW = KS * 32 + 8;          // a latent in LDS, with 16 bytes between rows so that 16 rows' words spread over the banks
  constexpr int SROW = KEYS + 4;            // a column's scores
  constexpr int OROW = KS * 32 + 4;         // a column's sums, at the end
  constexpr int NB = KS / 4;                // blocks of 128 channels
  constexpr int UNITS = NB * CT, UPW = (UNITS + 3) / 4;   // units, and how many a wave takes
  constexpr int PARTS = UNITS >= 4 ? 1 : 4 / UNITS;       // waves that share a unit
  constexpr int RUNS = KEYS / 32 / PARTS;   // runs of 32 keys a wave takes of a step
  static_assert(UPW == 1 || NB == 4, "a wave's units share their block");
  static_assert(CT * 16 * OROW * 4 <= KEYS * ROW * 2, "the sums take the latents' place");
  __shared__ __align__(16) bf16 cbuf[KEYS * ROW];
  __shared__ __align__(16) float sbuf[CT * 16 * SROW];
  __shared__ float lbuf[CT * 16];
  const int row = blockIdx.z, hg = blockIdx.y, split = blockIdx.x;
  const int pos = positions[row];
  const int c0 = split * chunk;
  if (c0 > pos) return;                     // the chunk holds no key of the request (the whole workgroup)
  const int last = min(c0 + chunk - 1, pos);
  const int lane = threadIdx.x & 63, j = lane & 15, c = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int32_t* table = tables + (size_t)row * table_stride;

  // Nothing is loaded behind a condition: lanes beyond the last key read the last key again (their scores are masked), pieces
  // beyond the latent's read its last one again (the queries hold zeros there, and such channels' sums go nowhere), columns
  // beyond the heads the last head.
  const int pieces = R / 8;
  bf16x8 kf[KT][KS];
  auto load_tile = [&](int kb) {
#pragma unroll
    for (int t = 0; t < KT; ++t) {
      const int key0 = min(kb + wave * 16 * KT + 16 * t, last & ~15);        // 16 keys in a row lie in one page
      const bf16* b = pages + (size_t)table[key0 / P] * P * R;
      const int slot = key0 % P + min(j, last - key0);
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        if (FULL)
          kf[t][ks] = load8_once(b + (size_t)(ks * 4 * P) * 8 + (c * P + slot) * 8);
        else
          kf[t][ks] = load8_once(b + (size_t)(min(ks * 4 + c, pieces - 1) * P + slot) * 8);
      }
    }
  };
  load_tile(c0);

  bf16x8 qf[CT][KS];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct) {
    const bf16* qr = q + ((size_t)row * H + min((hg * CT + ct) * 16 + j, H - 1)) * R + 8 * c;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      if (FULL)
        qf[ct][ks] = load8(qr + ks * 32);
      else
        qf[ct][ks] = ks * 32 + 8 * c < R ? load8(qr + ks * 32) : zero8();
    }
  }
  f32x4 acc[UPW][8];
  float m[UPW], l[UPW];
#pragma unroll
  for (int u = 0; u < UPW; ++u) {
    m[u] = -INFINITY;
    l[u] = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[u][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  // this wave's units: block of channels `block` (pieces 16 block .. 16 block + 15) with column tile (unit + 4 u) / NB; its part
  // of a unit's runs of keys
  const int unit = wave % (UNITS < 4 ? UNITS : 4), part = wave / (UNITS < 4 ? UNITS : 4);
  const int block = unit % NB;

  for (int kb = c0; kb <= last; kb += KEYS) {
    f32x4 s[KT][CT];
#pragma unroll
    for (int t = 0; t < KT; ++t)
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) s[t][ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int t = 0; t < KT; ++t)
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) s[t][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[t][ks], qf[ct][ks], s[t][ct], 0, 0, 0);
    // every wave is through with the last step's latents and scores
    if (kb > c0) asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
#pragma unroll
    for (int t = 0; t < KT; ++t) {
      const int k0 = (wave * KT + t) * 16;
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
#pragma unroll
        for (int r = 0; r < 4; ++r) s[t][ct][r] = kb + k0 + 4 * c + r <= last ? s[t][ct][r] * scale2 : -INFINITY;
        *reinterpret_cast<f32x4*>(&sbuf[(ct * 16 + j) * SROW + k0 + 4 * c]) = s[t][ct];
      }
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) *reinterpret_cast<bf16x8*>(&cbuf[(k0 + j) * ROW + (ks * 4 + c) * 8]) = kf[t][ks];
    }
    if (kb + KEYS <= last) load_tile(kb + KEYS);
    // what this wave wrote is in LDS; its loads on their way go on
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
    bf16x8 pf[UPW][RUNS];
#pragma unroll
    for (int u = 0; u < UPW; ++u) {
      const float* sc = &sbuf[((unit + 4 * u) / NB * 16 + j) * SROW + 8 * c];
      float mx = -INFINITY;
#pragma unroll
      for (int g = 0; g < KEYS / 32; ++g) {
        const f32x4 a = *reinterpret_cast<const f32x4*>(sc + 32 * g), b = *reinterpret_cast<const f32x4*>(sc + 32 * g + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) mx = fmaxf(mx, fmaxf(a[e], b[e]));
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
      mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
      const float m_new = fmaxf(m[u], mx);   // (a step holds at least one key: finite)
      const float alpha = __builtin_amdgcn_exp2f(m[u] - m_new);
      float sum = 0.f;
#pragma unroll
      for (int g = 0; g < RUNS; ++g) {
        const float* sp = sc + 32 * (g * PARTS + part);
        const f32x4 a = *reinterpret_cast<const f32x4*>(sp), b = *reinterpret_cast<const f32x4*>(sp + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float w0 = __builtin_amdgcn_exp2f(a[e] - m_new), w1 = __builtin_amdgcn_exp2f(b[e] - m_new);
          sum += w0 + w1;
          pf[u][g][e] = (bf16)w0;
          pf[u][g][4 + e] = (bf16)w1;
        }
      }
      l[u] = l[u] * alpha + sum;
      m[u] = m_new;
      if (__any(alpha != 1.f)) {
#pragma unroll
        for (int i = 0; i < 8; ++i)
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[u][i][r] *= alpha;
      }
    }
#pragma unroll
    for (int g = 0; g < RUNS; ++g) {
      uint32_t in[8][4];   // key 8 c + e of the run, channels 8 piece .. + 7
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const uint4 v = *reinterpret_cast<const uint4*>(&cbuf[(32 * (g * PARTS + part) + 8 * c + e) * ROW + (block * 16 + j) * 8]);
        in[e][0] = v.x, in[e][1] = v.y, in[e][2] = v.z, in[e][3] = v.w;
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        union {
          uint32_t w[4];
          bf16x8 v;
        } af;   // channel 8 piece + i, keys 8 c .. 8 c + 7
#pragma unroll
        for (int k = 0; k < 4; ++k)
          af.w[k] = __builtin_amdgcn_perm(in[2 * k + 1][i / 2], in[2 * k][i / 2], (i & 1) ? 0x07060302u : 0x05040100u);
#pragma unroll
        for (int u = 0; u < UPW; ++u) acc[u][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af.v, pf[u][g], acc[u][i], 0, 0, 0);
      }
    }
  }
  // the sums go out through LDS, so that a column's channels leave in whole lines; the waves of a unit add theirs up in order
  float* obuf = reinterpret_cast<float*>(cbuf);
#pragma unroll
  for (int turn = 0; turn < PARTS; ++turn) {
    __syncthreads();
    if (part != turn) continue;
#pragma unroll
    for (int u = 0; u < UPW; ++u) {
      const int col = (unit + 4 * u) / NB * 16 + j;
      float total = l[u] + __shfl_xor(l[u], 16, kWave);
      total += __shfl_xor(total, 32, kWave);
      if (block == 0 && c == 0) {
        lbuf[col] = turn == 0 ? total : lbuf[col] + total;
        const int head = hg * CT * 16 + col;
        if (turn == 0 && head < H) ws_ml[(((size_t)row * H + head) * splits + split) * 2] = m[u];   // (the same in every part)
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float* o = obuf + col * OROW + (block * 16 + 4 * c + r) * 8;
        f32x4 a, b;
#pragma unroll
        for (int e = 0; e < 4; ++e) a[e] = acc[u][e][r], b[e] = acc[u][4 + e][r];
        if (turn > 0) {
          a += *reinterpret_cast<const f32x4*>(o);
          b += *reinterpret_cast<const f32x4*>(o + 4);
        }
        *reinterpret_cast<f32x4*>(o) = a;
        *reinterpret_cast<f32x4*>(o + 4) = b;
      }
    }
  }
  __syncthreads();
  const int heads = min(CT * 16, H - hg * CT * 16);
  float* cells = ws_acc + (((size_t)row * H + hg * CT * 16) * splits + split) * R;   // a head's are splits * R apart
  for (int col = wave; col < heads; col += 4) {
#pragma unroll
    for (int i = 0; i < (KS * 8 + 63) / 64; ++i) {
      const int ch = (lane + 64 * i) * 4;
      if (ch < R) *reinterpret_cast<f32x4*>(cells + (size_t)col * splits * R + ch) = *reinterpret_cast<const f32x4*>(obuf + col * OROW + ch);
    }
  }
  if ((int)threadIdx.x < heads) ws_ml[(((size_t)row * H + hg * CT * 16 + threadIdx.x) * splits + split) * 2 + 1] = lbuf[threadIdx.x];
}

// Any sizes and types: 256 threads, a thread a key for the scores and a thread a channel (and every 256th after it) for the sums.
template <typename T>
__global__ __launch_bounds__(256) void latent_decode_plain_kernel(const T* __restrict__ q, const T* __restrict__ pages,
                                                                  const int32_t* __restrict__ tables, int table_stride,
                                                                  const int32_t* __restrict__ positions,
                                                                  const int32_t* __restrict__ tok_seq, int H, int R, int P,
                                                                  float scale2, int chunk, int splits, float* __restrict__ ws_acc,
                                                                  float* __restrict__ ws_ml) {
  extern __shared__ float smem[];
  float* qs = smem;            // [R]
  float* es = smem + R;        // [256]
  float* scratch = es + 256;   // [17]
  const int t = blockIdx.y / H, h = blockIdx.y % H, split = blockIdx.x, tid = threadIdx.x;
  const int pos = positions[t], c0 = split * chunk;
  if (c0 > pos) return;
  const int last = min(c0 + chunk - 1, pos);
  const int32_t* table = tables + (size_t)tok_seq[t] * table_stride;
  const int piece = key_piece(R);
  for (int r = tid; r < R; r += 256) qs[r] = to_f(q[((size_t)t * H + h) * R + r]);
  __syncthreads();
  float m = -INFINITY, l = 0.f, acc[kMaxRank / 256];
#pragma unroll
  for (int i = 0; i < kMaxRank / 256; ++i) acc[i] = 0.f;
  for (int k0 = c0; k0 <= last; k0 += 256) {
    const int key = k0 + tid;
    float s = -INFINITY;
    if (key <= last) {
      const T* page = pages + (size_t)table[key / P] * P * R;
      float dot = 0.f;
      for (int r0 = 0; r0 < R; r0 += piece) {
        const T* kr = page + key_offset(key % P, r0, P, piece);
        for (int e = 0; e < piece; ++e) dot = fmaf(qs[r0 + e], to_f(kr[e]), dot);
      }
      s = dot * scale2;
    }
    const float m_new = fmaxf(m, block_max(s, scratch));
    const float e = key <= last ? exp2f(s - m_new) : 0.f;
    es[tid] = e;
    const float alpha = exp2f(m - m_new);
    l = fmaf(l, alpha, block_sum(e, scratch));   // (also orders the writes of es before the reads below)
    m = m_new;
#pragma unroll
    for (int i = 0; i < kMaxRank / 256; ++i) acc[i] *= alpha;
    const int top = min(k0 + 255, last);
    for (int k = k0; k <= top; ++k) {
      const T* page = pages + (size_t)table[k / P] * P * R;
      const float w = es[k - k0];
#pragma unroll
      for (int i = 0; i < kMaxRank / 256; ++i) {
        const int r = tid + 256 * i;
        if (r < R) acc[i] = fmaf(w, to_f(page[key_offset(k % P, r, P, piece)]), acc[i]);
      }
    }
    __syncthreads();   // es is written again
  }
  const size_t cell = ((size_t)t * H + h) * splits + split;
  if (tid == 0) {
    ws_ml[cell * 2] = m;
    ws_ml[cell * 2 + 1] = l;
  }
#pragma unroll
  for (int i = 0; i < kMaxRank / 256; ++i)
    if (tid + 256 * i < R) ws_acc[cell * R + tid + 256 * i] = acc[i];
}

// ------------------------------------------------------------------------------------------------ latent_finish
// A workgroup a (token, head): uv [H * hc, R] (the first vdim rows of a head), gate [n, ldg].  WORDS (bfloat16, R a multiple of
// 8): sixteen lanes a channel of the value, 16 bytes of a row of W_uv a lane; the first 64 rows' first 512 channels are asked for
// before anything else.
template <typename T, bool WORDS>
__global__ __launch_bounds__(256) void latent_finish_kernel(const float* __restrict__ ws_acc, const float* __restrict__ ws_ml,
                                                            const int32_t* __restrict__ positions, int chunk, int splits,
                                                            const float* __restrict__ sinks, const T* __restrict__ uv, int hc,
                                                            const T* __restrict__ gate, int ldg, T* __restrict__ out, int ldo, int H,
                                                            int R, int vdim) {
  __shared__ float weight[kMaxSplits];
  __shared__ __align__(16) float o[kMaxRank];
  __shared__ __align__(16) float half_sums[1024];
  const int t = blockIdx.x / H, h = blockIdx.x % H, tid = threadIdx.x;
  const int g16 = tid / 16, l16 = tid % 16;
  const T* w = uv + (size_t)h * hc * R;
  bf16x8 early[4][4];
  if constexpr (WORDS) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const int d = g16 + 16 * i, p = l16 + 16 * k;
        early[i][k] = (d < vdim && p * 8 < R) ? load8(w + (size_t)d * R + 8 * p) : zero8();
      }
  }
  const size_t cell0 = ((size_t)t * H + h) * splits;
  // four channels a thread; where that leaves threads over, groups of them take the chunks in turn
  const bool by_quads = R % 4 == 0 && R <= 1024;
  const int quads = by_quads ? R / 4 : 256, groups = 256 / quads, group = tid / quads, q4 = (tid % quads) * 4;
  const int count = min(positions[t] / chunk + 1, splits);   // chunks that hold keys
  // every wave finds the maximum and the sum for itself (a lane a chunk, and every 64th after it): no barriers
  const int lane = tid % kWave;
  float m_of[kMaxSplits / kWave], l_of[kMaxSplits / kWave], top = -INFINITY, total = 0.f;
#pragma unroll
  for (int i = 0; i < kMaxSplits / kWave; ++i) {
    const int k = lane + kWave * i;
    m_of[i] = k < count ? ws_ml[(cell0 + k) * 2] : -INFINITY;
    l_of[i] = k < count ? ws_ml[(cell0 + k) * 2 + 1] : 0.f;
    top = fmaxf(top, m_of[i]);
  }
  top = wave_max(top);
#pragma unroll
  for (int i = 0; i < kMaxSplits / kWave; ++i) {
    const float f = m_of[i] == -INFINITY ? 0.f : exp2f(m_of[i] - top);
    if (tid < kWave) weight[lane + kWave * i] = f;
    total = fmaf(f, l_of[i], total);
  }
  total = wave_sum(total);
  if (sinks) total += exp2f(fmaf(sinks[h], kLog2e, -top));
  const float inv = 1.0f / total;
  __syncthreads();
  if (by_quads) {
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
    if (group < groups) {
#pragma unroll 8
      for (int k = group; k < count; k += groups) s += *reinterpret_cast<const f32x4*>(ws_acc + (cell0 + k) * R + q4) * weight[k];
      *reinterpret_cast<f32x4*>(&half_sums[group * R + q4]) = s;
    }
    __syncthreads();
    for (int r = tid; r < R; r += 256) {
      float v = 0.f;
      for (int k = 0; k < groups; ++k) v += half_sums[k * R + r];
      o[r] = v * inv;
    }
  } else {
    for (int r = tid; r < R; r += 256) {
      float s = 0.f;
      for (int k = 0; k < count; ++k) s = fmaf(ws_acc[(cell0 + k) * R + r], weight[k], s);
      o[r] = s * inv;
    }
  }
  __syncthreads();
  auto finish = [&](int d, float s) {   // the sixteen lanes' sums of channel d
#pragma unroll
    for (int off = 8; off >= 1; off >>= 1) s += __shfl_xor(s, off, 16);
    if (l16 == 0 && d < vdim) {
      s = s / (1.0f + expf(-to_f(gate[(size_t)t * ldg + (size_t)h * vdim + d])));
      out[(size_t)t * ldo + (size_t)h * vdim + d] = from_f<T>(s);
    }
  };
  auto dot8 = [&](const bf16x8& v, int p, float s) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(&o[8 * p]), b = *reinterpret_cast<const f32x4*>(&o[8 * p + 4]);
#pragma unroll
    for (int e = 0; e < 4; ++e) s = fmaf((float)v[e], a[e], s);
#pragma unroll
    for (int e = 0; e < 4; ++e) s = fmaf((float)v[4 + e], b[e], s);
    return s;
  };
  if constexpr (WORDS) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = g16 + 16 * i;
      float s = 0.f;
#pragma unroll
      for (int k = 0; k < 4; ++k)
        if ((l16 + 16 * k) * 8 < R) s = dot8(early[i][k], l16 + 16 * k, s);
      if (d < vdim)
        for (int p = l16 + 64; p < R / 8; p += 16) s = dot8(load8(w + (size_t)d * R + 8 * p), p, s);
      finish(d, s);
    }
    for (int d = g16 + 64; d < vdim; d += 16) {
      float s = 0.f;
      for (int p = l16; p < R / 8; p += 16) s = dot8(load8(w + (size_t)d * R + 8 * p), p, s);
      finish(d, s);
    }
  } else {
    for (int d = g16; d < vdim; d += 16) {
      float s = 0.f;
      for (int r = l16; r < R; r += 16) s = fmaf(to_f(w[(size_t)d * R + r]), o[r], s);
      finish(d, s);
    }
  }
}

// ------------------------------------------------------------------------------------------------ scratch pages of portions
// Requests first .. first + count - 1 of the step; a request's context is pos0 + q_len tokens.  table [*, stride] (rows by
// request) receives the scratch pages in order, source [total][2] the (request, page of its context) behind each.
__global__ __launch_bounds__(256) void latent_tables_kernel(const int32_t* __restrict__ q_len, const int32_t* __restrict__ pos0, int first,
                                                            int count, int P, int32_t* __restrict__ table, int stride,
                                                            int32_t* __restrict__ source, int total) {
  int base = 0;
  for (int s = first; s < first + count; ++s) {
    const int pages = (pos0[s] + q_len[s] + P - 1) / P;
    for (int i = threadIdx.x; i < pages && i < stride && base + i < total; i += 256) {
      table[(size_t)s * stride + i] = base + i;
      source[2 * (base + i)] = s;
      source[2 * (base + i) + 1] = i;
    }
    base += pages;
  }
}

// A workgroup a scratch page: its tokens' latents as rows [P][R], zeros behind the context's end.
template <typename T>
__global__ __launch_bounds__(256) void latent_gather_kernel(const T* __restrict__ pages, const int32_t* __restrict__ tables,
                                                            int table_stride, const int32_t* __restrict__ source,
                                                            const int32_t* __restrict__ q_len, const int32_t* __restrict__ pos0, int P,
                                                            int R, T* __restrict__ out) {
  const int s = source[2 * blockIdx.x], i = source[2 * blockIdx.x + 1];
  const int valid = min(P, pos0[s] + q_len[s] - i * P);
  const T* page = pages + (size_t)tables[(size_t)s * table_stride + i] * P * R;
  T* rows = out + (size_t)blockIdx.x * P * R;
  if constexpr (std::is_same<T, bf16>::value) {
    if (R % 8 == 0) {
      const int pieces = R / 8;
      for (int u = threadIdx.x; u < P * pieces; u += 256) {
        const int slot = u / pieces, p = u % pieces;
        *reinterpret_cast<bf16x8*>(rows + (size_t)slot * R + 8 * p) = slot < valid ? load8(page + ((size_t)p * P + slot) * 8) : zero8();
      }
      return;
    }
  }
  const int piece = key_piece(R);
  for (int u = threadIdx.x; u < P * R; u += 256) {
    const int slot = u / R, r = u % R;
    rows[u] = slot < valid ? page[key_offset(slot, r, P, piece)] : from_f<T>(0.f);
  }
}

// Rows [n][H key heads | H value heads] of hc columns; row r goes to slot r % P of scratch page r / P.  A workgroup (16 rows,
// head): keys word by word into their pieces, values turned in LDS.
__global__ __launch_bounds__(256) void latent_expand_words_kernel(const bf16* __restrict__ kv, int ld, bf16* __restrict__ k_pages,
                                                                  bf16* __restrict__ v_pages, int H, int hc, int P) {
  extern __shared__ uint32_t tile[];   // [16][hc / 2 + 1]
  const int r0 = blockIdx.x * 16, h = blockIdx.y, page = r0 / P, slot0 = r0 % P;
  const int words = hc / 8, pitch = hc / 2 + 1;
  bf16* kb = k_pages + ((size_t)page * H + h) * hc * P;
  bf16* vb = v_pages + ((size_t)page * H + h) * hc * P;
  for (int u = threadIdx.x; u < 16 * words; u += 256) {
    const int slot = u / words, p = u % words;
    const uint4 v = *reinterpret_cast<const uint4*>(kv + (size_t)(r0 + slot) * ld + (size_t)(H + h) * hc + 8 * p);
    uint32_t* d = tile + slot * pitch + 4 * p;
    d[0] = v.x, d[1] = v.y, d[2] = v.z, d[3] = v.w;
  }
  for (int u = threadIdx.x; u < 16 * words; u += 256) {
    const int p = u / 16, slot = u % 16;
    *reinterpret_cast<bf16x8*>(kb + ((size_t)p * P + slot0 + slot) * 8) = load8(kv + (size_t)(r0 + slot) * ld + (size_t)h * hc + 8 * p);
  }
  __syncthreads();
  for (int u = threadIdx.x; u < hc * 2; u += 256) {   // (channel, half of the 16 slots)
    const int d = u / 2, s0 = (u % 2) * 8;
    uint4 w;
    uint32_t* wp = &w.x;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const uint32_t lo = tile[(s0 + 2 * k) * pitch + d / 2], hi = tile[(s0 + 2 * k + 1) * pitch + d / 2];
      wp[k] = (d & 1) ? __builtin_amdgcn_perm(hi, lo, 0x07060302u) : __builtin_amdgcn_perm(hi, lo, 0x05040100u);
    }
    *reinterpret_cast<uint4*>(vb + (size_t)d * P + slot0 + s0) = w;
  }
}

template <typename T>
__global__ void latent_expand_kernel(const T* __restrict__ kv, int ld, T* __restrict__ k_pages, T* __restrict__ v_pages, int H, int hc,
                                     int P, long long count) {
  const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
  if (idx >= count) return;
  const int d = (int)(idx % hc), h = (int)(idx / hc % H);
  const long long r = idx / hc / H;
  const size_t base = ((size_t)(r / P) * H + h) * hc * P;
  const int slot = (int)(r % P);
  k_pages[base + key_offset(slot, d, P, key_piece(hc))] = kv[(size_t)r * ld + (size_t)h * hc + d];
  v_pages[base + (size_t)d * P + slot] = kv[(size_t)r * ld + (size_t)(H + h) * hc + d];
}

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

// in [n, ld] of `dtype`, the latent in the first R columns; pages [pages][R / piece][P][piece].
extern "C" int gb_latent_store(const void* in, int dtype, int ld, const float* gamma, float eps, const int32_t* slots, void* pages,
                               int page_size, int n, int R, hipStream_t stream) {
  GB_REQUIRE(n >= 0 && R > 0 && ld >= R && page_size > 0 && in && gamma && slots && pages, "latent_store: bad sizes n=%d R=%d ld=%d", n, R, ld);
  if (n == 0) return 0;
  const int words = dtype == kBF16 && R % 8 == 0 && ld % 8 == 0 && words16(in) && words16(pages);
  GB_BY_DTYPE(dtype, "latent_store",
              hipLaunchKernelGGL(latent_store_kernel<TT>, dim3((unsigned)((n + 3) / 4)), dim3(256), 0, stream, (const TT*)in, ld, gamma,
                                 eps, slots, (TT*)pages, page_size, n, R, words))
  return launched("latent_store");
}

// q [n, ldq]: H heads of hc columns; uk [H * hc, R]; uk_t [H, R, hc] or nullptr (then, and in 32-bit, the plain kernel); out
// [n, H * R].
extern "C" int gb_latent_absorb(const void* q, int dtype, int ldq, const void* uk, const void* uk_t, int hc, int dim, void* out, int n,
                                int H, int R, hipStream_t stream) {
  GB_REQUIRE(n >= 0 && H > 0 && R > 0 && dim > 0 && hc >= dim && ldq >= H * hc && q && uk && out, "latent_absorb: bad sizes n=%d heads=%d R=%d dim=%d of %d", n, H, R, dim, hc);
  if (n == 0) return 0;
  if (dtype == kBF16 && uk_t && R % 8 == 0 && hc % 8 == 0 && ldq % 8 == 0 && words16(q) && words16(uk_t) && words16(out) && H <= 65535 && n <= 65535 * 16) {
    const dim3 grid((unsigned)((R + 63) / 64), (unsigned)H, (unsigned)((n + 15) / 16));
    hipLaunchKernelGGL(latent_absorb_kernel, grid, dim3(64), 0, stream, (const bf16*)q, ldq, (const bf16*)uk_t, hc, (bf16*)out, n, H, R);
    return launched("latent_absorb");
  }
  const long long count = (long long)n * H * R;
  GB_REQUIRE(grid_fits(count, 256), "latent_absorb: too many elements");
  GB_BY_DTYPE(dtype, "latent_absorb",
              hipLaunchKernelGGL(latent_absorb_plain_kernel<TT>, dim3((unsigned)((count + 255) / 256)), dim3(256), 0, stream, (const TT*)q,
                                 ldq, (const TT*)uk, hc, dim, (TT*)out, count, H, R))
  return launched("latent_absorb");
}

// gb_latent_store and gb_latent_absorb of the first n_q rows in one launch: rows [n, ld] bfloat16 hold H query heads of hc columns
// and the latent from column c_col on; R and hc multiples of 8, everything aligned.
extern "C" int gb_latent_store_absorb(const void* rows, int ld, int c_col, const float* gamma, float eps, const int32_t* slots, void* pages,
                                      int page_size, int n, const void* uk_t, int hc, void* out, int n_q, int H, int R,
                                      hipStream_t stream) {
  GB_REQUIRE(n_q > 0 && n >= n_q && H > 0 && H < 65535 && R > 0 && R % 8 == 0 && hc > 0 && hc % 8 == 0 && c_col >= H * hc && ld >= c_col + R,
             "latent_store_absorb: bad sizes n=%d of %d heads=%d of %d R=%d", n_q, n, H, hc, R);
  GB_REQUIRE(ld % 8 == 0 && c_col % 8 == 0 && words16(rows) && words16(pages) && words16(uk_t) && words16(out) && gamma && slots && page_size > 0 && n_q <= 65535 * 16,
             "latent_store_absorb: operands must be 16-byte aligned rows");
  const dim3 grid((unsigned)((R + 63) / 64), (unsigned)(H + 1), (unsigned)((n_q + 15) / 16));
  hipLaunchKernelGGL(latent_store_absorb_kernel, grid, dim3(64), 0, stream, (const bf16*)rows, ld, c_col, gamma, eps, slots, (bf16*)pages,
                     page_size, n, (const bf16*)uk_t, hc, (bf16*)out, n_q, H, R);
  return launched("latent_store_absorb");
}

// Whether the matrix-core kernel takes latents of R channels in pages of P tokens.
extern "C" int gb_latent_decode_takes(int R, int P) { return R >= 8 && R % 8 == 0 && R <= 512 && P >= 16 && P % 16 == 0; }

// q [n, H * R] (row t is request t's single token for the matrix-core kernel; any rows with tok_seq for the plain one), pages as
// gb_latent_store writes them, ws_acc [n, H, splits, R] and ws_ml [n, H, splits, 2] float32 with splits = ceil(longest context /
// chunk); only the chunks that hold keys of a row are written.
extern "C" int gb_latent_decode(const void* q, int dtype, const void* pages, const int32_t* tables, int table_stride,
                                const int32_t* positions, const int32_t* tok_seq, int n, int H, int R, int P, float scale, int chunk,
                                int splits, float* ws_acc, float* ws_ml, int plain, hipStream_t stream) {
  GB_REQUIRE(n >= 0 && H > 0 && R > 0 && R <= kMaxRank && P > 0 && table_stride > 0, "latent_decode: bad sizes n=%d heads=%d R=%d (at most %d)", n, H, R, kMaxRank);
  GB_REQUIRE(chunk > 0 && splits >= 1 && splits <= kMaxSplits, "latent_decode: %d chunks of a context (at most %d)", splits, kMaxSplits);
  GB_REQUIRE(q && pages && tables && positions && ws_acc && ws_ml, "latent_decode: operands are missing");
  if (n == 0) return 0;
  const float scale2 = scale * kLog2e;
  if (!plain) {
    GB_REQUIRE(dtype == kBF16 && gb_latent_decode_takes(R, P), "latent_decode: R=%d in pages of %d goes through the plain kernel", R, P);
    GB_REQUIRE(chunk % 128 == 0 && n <= 65535 && words16(q) && words16(pages) && words16(ws_acc), "latent_decode: chunks of whole 128 keys, aligned operands");
    const int ct = H > 16 ? 2 : 1;
    const dim3 grid((unsigned)splits, (unsigned)((H + 16 * ct - 1) / (16 * ct)), (unsigned)n);
#define GB_LATENT_AS(KS, CT, FULL)                                                                                              \
  if (ct == CT && (R == KS * 32) == FULL)                                                                                       \
    hipLaunchKernelGGL((latent_decode_kernel<KS, CT, FULL>), grid, dim3(256), 0, stream, (const bf16*)q, (const bf16*)pages,     \
                       tables, table_stride, positions, H, R, P, scale2, chunk, splits, ws_acc, ws_ml);
#define GB_LATENT(KS) GB_LATENT_AS(KS, 1, true) GB_LATENT_AS(KS, 1, false) GB_LATENT_AS(KS, 2, true) GB_LATENT_AS(KS, 2, false)
    if (R <= 128) {
      GB_LATENT(4)
    } else if (R <= 256) {
      GB_LATENT(8)
    } else {
      GB_LATENT(16)
    }
#undef GB_LATENT_AS
#undef GB_LATENT
    return launched("latent_decode");
  }
  GB_REQUIRE(tok_seq, "latent_decode: the plain kernel needs the rows' requests");
  const int rows_max = 65535 / H;   // (grid.y)
  GB_REQUIRE(rows_max >= 1, "latent_decode: %d heads", H);
  for (int first = 0; first < n; first += rows_max) {
    const int rows = n - first < rows_max ? n - first : rows_max;
    const dim3 grid((unsigned)splits, (unsigned)(rows * H));
    const size_t lds = (size_t)(R + 256 + 17) * sizeof(float);
    GB_BY_DTYPE(dtype, "latent_decode",
                hipLaunchKernelGGL(latent_decode_plain_kernel<TT>, grid, dim3(256), lds, stream, (const TT*)q + (size_t)first * H * R,
                                   (const TT*)pages, tables, table_stride, positions + first, tok_seq + first, H, R, P, scale2, chunk,
                                   splits, ws_acc + (size_t)first * H * splits * R, ws_ml + (size_t)first * H * splits * 2))
  }
  return launched("latent_decode (plain)");
}

// The partial results of gb_latent_decode to out [n, ldo] of `dtype`: H heads of vdim columns, gated.
extern "C" int gb_latent_finish(const float* ws_acc, const float* ws_ml, const int32_t* positions, int chunk, int splits,
                                const float* sinks, const void* uv, int hc, const void* gate, int ldg, void* out, int ldo, int dtype,
                                int n, int H, int R, int vdim, hipStream_t stream) {
  GB_REQUIRE(n >= 0 && H > 0 && R > 0 && R <= kMaxRank && vdim > 0 && hc >= vdim && ldo >= H * vdim && gate && ldg >= H * vdim,
             "latent_finish: bad sizes n=%d heads=%d R=%d vdim=%d", n, H, R, vdim);
  GB_REQUIRE(chunk > 0 && splits >= 1 && splits <= kMaxSplits && ws_acc && ws_ml && positions && uv && out, "latent_finish: %d chunks, or operands are missing", splits);
  if (n == 0) return 0;
  GB_REQUIRE((long long)n * H < (1ll << 31), "latent_finish: too many (token, head) pairs");
  GB_REQUIRE(R % 4 != 0 || words16(ws_acc), "latent_finish: the partial sums must be 16-byte aligned");
#define GB_FINISH(T, WORDS)                                                                                                     \
  hipLaunchKernelGGL((latent_finish_kernel<T, WORDS>), dim3((unsigned)(n * H)), dim3(256), 0, stream, ws_acc, ws_ml, positions, \
                     chunk, splits, sinks, (const T*)uv, hc, (const T*)gate, ldg, (T*)out, ldo, H, R, vdim)
  if (dtype == kBF16 && R % 8 == 0 && words16(uv))
    GB_FINISH(bf16, true);
  else if (dtype == kBF16)
    GB_FINISH(bf16, false);
  else if (dtype == kF32)
    GB_FINISH(float, false);
  else
    return fail("latent_finish: unknown dtype %d", dtype);
#undef GB_FINISH
  return launched("latent_finish");
}

extern "C" int gb_latent_tables(const int32_t* q_len, const int32_t* pos0, int first, int count, int P, int32_t* table, int stride,
                                int32_t* source, int total, hipStream_t stream) {
  GB_REQUIRE(first >= 0 && count >= 0 && P > 0 && stride > 0 && total >= 0 && q_len && pos0 && table && source, "latent_tables: bad sizes");
  if (count == 0) return 0;
  hipLaunchKernelGGL(latent_tables_kernel, dim3(1), dim3(256), 0, stream, q_len, pos0, first, count, P, table, stride, source, total);
  return launched("latent_tables");
}

// out [total * P, R]
extern "C" int gb_latent_gather(const void* pages, int dtype, const int32_t* tables, int table_stride, const int32_t* source,
                                const int32_t* q_len, const int32_t* pos0, int P, int R, int total, void* out, hipStream_t stream) {
  GB_REQUIRE(P > 0 && R > 0 && total >= 0 && pages && tables && source && q_len && pos0 && out, "latent_gather: bad sizes");
  GB_REQUIRE(R % 8 != 0 || (words16(pages) && words16(out)), "latent_gather: operands must be 16-byte aligned");
  if (total == 0) return 0;
  GB_BY_DTYPE(dtype, "latent_gather",
              hipLaunchKernelGGL(latent_gather_kernel<TT>, dim3((unsigned)total), dim3(256), 0, stream, (const TT*)pages, tables,
                                 table_stride, source, q_len, pos0, P, R, (TT*)out))
  return launched("latent_gather");
}

// kv [total * P, ld]: H key heads, then H value heads, of hc columns; k_pages [total, H, hc / piece, P, piece], v_pages [total, H,
// hc, P].
extern "C" int gb_latent_expand(const void* kv, int dtype, int ld, void* k_pages, void* v_pages, int H, int hc, int P, int total,
                                hipStream_t stream) {
  GB_REQUIRE(H > 0 && hc > 0 && P > 0 && total >= 0 && ld >= 2 * H * hc && kv && k_pages && v_pages, "latent_expand: bad sizes heads=%d of %d", H, hc);
  if (total == 0) return 0;
  if (dtype == kBF16 && hc % 8 == 0 && P % 16 == 0 && ld % 8 == 0 && words16(kv) && words16(k_pages) && words16(v_pages) && H <= 65535) {
    const dim3 grid((unsigned)(total * (P / 16)), (unsigned)H);
    hipLaunchKernelGGL(latent_expand_words_kernel, grid, dim3(256), (size_t)16 * (hc / 2 + 1) * 4, stream, (const bf16*)kv, ld,
                       (bf16*)k_pages, (bf16*)v_pages, H, hc, P);
    return launched("latent_expand");
  }
  const long long count = (long long)total * P * H * hc;
  GB_REQUIRE(grid_fits(count, 256), "latent_expand: too many elements");
  GB_BY_DTYPE(dtype, "latent_expand",
              hipLaunchKernelGGL(latent_expand_kernel<TT>, dim3((unsigned)((count + 255) / 256)), dim3(256), 0, stream, (const TT*)kv, ld,
                                 (TT*)k_pages, (TT*)v_pages, H, hc, P, count))
  return launched("latent_expand");
}

// the launches of a layer can be recorded and made again for the layers like it (common.h)
GB_TAPED(gb_latent_store)
GB_TAPED(gb_latent_absorb)
GB_TAPED(gb_latent_store_absorb)
GB_TAPED(gb_latent_decode)
GB_TAPED(gb_latent_finish)
GB_TAPED(gb_latent_tables)
GB_TAPED(gb_latent_gather)
GB_TAPED(gb_latent_expand)
