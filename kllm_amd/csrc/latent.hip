// Attention through low-rank latents.  Per token one vector is cached for all heads: the
// normalised latent c [rank] followed by one rotated key part [dr].  A head's key is
// [W_uk,h c | rotated part] and its value W_uv,h c, so with the query's unrotated part folded
// through W_uk,h (q' = W_uk,h^T q, [rank]) the score is q' . c + q_rot . k_rot, the weighted
// sum over the keys is taken of c itself, and W_uv,h is applied once to that sum:
//
//   latent_kv_append   sums of W_dkv h -> RMS norm (weights) of the first rank, rotation of the
//                      last dr (halves paired), appended to the pages (one row of rank + dr a slot)
//   latent_query       sums of W_uq c_q -> per head [W_uk,h^T q_h | rotated q_h], rank + dr wide
//   attn_latent        one workgroup a (token, head): online softmax over 256 keys at a time,
//                      the values being the first rank elements of the cached rows; with a window
//                      the last `window` keys only (pages behind it may be gone)
//   latent_out         per head W_uv,h times the attended latent, times sigmoid of the gate's sums
//                      (one gate an element, or one a head)
//
// Scores, softmax, norms and rotation are 32-bit; the cached rows, the folded queries and the
// attended latents are stored in the compute type.
//
// A page holds its slots' rows [slot][rank + dr] and then the latents once more, transposed
// [rank][slot]: the weighted sum over the keys runs along the slots, and the matrix cores want
// the dimension that is summed over contiguous.  attn_latent has two kernels: one workgroup a
// (token, head) in 32-bit arithmetic for every size and type, and, in bfloat16 for ranks in
// steps of 16 and rows in steps of 8, one on the matrix cores (below).
#include <math.h>
#include <stdint.h>

#include "common.hpp"
#include "kllm_kernels.h"

namespace kllm {

constexpr int kLatThreads = 256;
constexpr int kLatMaxRow = 1024;       // rank + dr of a cached row
constexpr int kLatMaxPer = kLatMaxRow / kLatThreads;

template <typename T>
__global__ __launch_bounds__(kLatThreads) void latent_kv_append_kernel(
    const float* __restrict__ dkv, int nsplit, long split_stride, const float* __restrict__ weight, float eps,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, T* __restrict__ cache,
    const int* __restrict__ positions, const int* __restrict__ span_of_token, const int* __restrict__ block_table,
    int max_pages, int page_size, int rank, int dr, long in_stride) {
  __shared__ float red[16];
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const int row = rank + dr, half = dr / 2;
  const float* in = dkv + t * in_stride;
  const int pos = positions[t];
  const long page = block_table[(long)span_of_token[t] * max_pages + pos / page_size];
  const long page_elems = (long)page_size * (row + rank);
  const int slot = pos % page_size;
  T* dst = cache + page * page_elems + (long)slot * row;
  T* dst_t = cache + page * page_elems + (long)page_size * row + slot;     // [rank][slot]
  float v[kLatMaxPer];
  float ss = 0.f;
#pragma unroll
  for (int q = 0; q < kLatMaxPer; ++q) {
    const int i = tid + q * kLatThreads;
    v[q] = 0.f;
    if (i < rank) {
      for (int s = 0; s < nsplit; ++s) v[q] += in[s * split_stride + i];
      ss = fmaf(v[q], v[q], ss);
    }
  }
  const float rstd = 1.f / sqrtf(block_sum(ss, red) / (float)rank + eps);
#pragma unroll
  for (int q = 0; q < kLatMaxPer; ++q) {
    const int i = tid + q * kLatThreads;
    if (i < rank) {
      const T c = from_f32<T>(v[q] * rstd * weight[i]);
      dst[i] = c;
      dst_t[(long)i * page_size] = c;
    }
  }
  for (int i = tid; i < half; i += kLatThreads) {
    float a = 0.f, b = 0.f;
    for (int s = 0; s < nsplit; ++s) {
      a += in[s * split_stride + rank + i];
      b += in[s * split_stride + rank + half + i];
    }
    const float c = cos_t[t * half + i], sn = sin_t[t * half + i];
    dst[rank + i] = from_f32<T>(a * c - b * sn);
    dst[rank + half + i] = from_f32<T>(b * c + a * sn);
  }
}

// out [n][r] = N(in row's r elements) * weight, the rows of `in` in_stride apart; one workgroup a row.
// PER > 0: rows of up to PER * kLatThreads elements, which a thread keeps in registers, so that its
// loads (a slice's all together) are one trip to memory each.
template <typename T, int PER>
__global__ __launch_bounds__(kLatThreads) void latent_norm_kernel(const float* __restrict__ in, int nsplit,
                                                                  long split_stride, long in_stride,
                                                                  const float* __restrict__ weight, float eps,
                                                                  T* __restrict__ out, int r) {
  __shared__ float red[16];
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const float* src = in + t * in_stride;
  float ss = 0.f;
  if constexpr (PER > 0) {
    float v[PER], w[PER];
#pragma unroll
    for (int j = 0; j < PER; ++j) {
      v[j] = 0.f;
      w[j] = weight[min(tid + kLatThreads * j, r - 1)];
    }
    for (int s = 0; s < nsplit; ++s)
#pragma unroll
      for (int j = 0; j < PER; ++j) v[j] += src[s * split_stride + min(tid + kLatThreads * j, r - 1)];
#pragma unroll
    for (int j = 0; j < PER; ++j)
      if (tid + kLatThreads * j < r) ss = fmaf(v[j], v[j], ss);
    const float rstd = 1.f / sqrtf(block_sum(ss, red) / (float)r + eps);
#pragma unroll
    for (int j = 0; j < PER; ++j)
      if (tid + kLatThreads * j < r) out[t * r + tid + kLatThreads * j] = from_f32<T>(v[j] * rstd * w[j]);
    return;
  }
  for (int i = tid; i < r; i += kLatThreads) {
    float v = 0.f;
    for (int s = 0; s < nsplit; ++s) v += src[s * split_stride + i];
    ss = fmaf(v, v, ss);
  }
  const float rstd = 1.f / sqrtf(block_sum(ss, red) / (float)r + eps);
  for (int i = tid; i < r; i += kLatThreads) {
    float v = 0.f;
    for (int s = 0; s < nsplit; ++s) v += src[s * split_stride + i];
    out[t * r + i] = from_f32<T>(v * rstd * weight[i]);
  }
}

// q: [nsplit][n][H * (d + dr)], a head laid out [d unrotated | dr rotated]; w_uk [H * d][rank].
template <typename T>
__global__ __launch_bounds__(kLatThreads) void latent_query_kernel(
    const float* __restrict__ q, int nsplit, long split_stride, const T* __restrict__ w_uk,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, T* __restrict__ out, int H, int d, int dr,
    int rank) {
  extern __shared__ float qh[];          // [d + dr]
  const long t = blockIdx.x;
  const int h = blockIdx.y, tid = threadIdx.x;
  const int hw = d + dr, half = dr / 2;
  const float* in = q + (t * H + h) * hw;
  for (int i = tid; i < hw; i += kLatThreads) {
    float v = 0.f;
    for (int s = 0; s < nsplit; ++s) v += in[s * split_stride + i];
    qh[i] = v;
  }
  __syncthreads();
  T* dst = out + (t * H + h) * (rank + dr);
  const T* w = w_uk + (long)h * d * rank;
  for (int r = tid; r < rank; r += kLatThreads) {
    float acc = 0.f;
    for (int i = 0; i < d; ++i) acc = fmaf(qh[i], to_f32(w[(long)i * rank + r]), acc);
    dst[r] = from_f32<T>(acc);
  }
  for (int i = tid; i < half; i += kLatThreads) {
    const float a = qh[d + i], b = qh[d + half + i];
    const float c = cos_t[t * half + i], sn = sin_t[t * half + i];
    dst[rank + i] = from_f32<T>(a * c - b * sn);
    dst[rank + half + i] = from_f32<T>(b * c + a * sn);
  }
}

template <typename T>
__global__ __launch_bounds__(kLatThreads) void attn_latent_kernel(
    const T* __restrict__ q, T* __restrict__ out, const T* __restrict__ cache, const int* __restrict__ positions,
    const int* __restrict__ span_of_token, const int* __restrict__ block_table, int max_pages, int page_size, int H,
    int row, int rank, float scale, int window) {
  __shared__ float qs[kLatMaxRow];
  __shared__ float ps[kLatThreads];
  __shared__ float red[16];
  const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const long page_elems = (long)page_size * (row + rank);
  const int len = positions[t] + 1;
  const int lo = first_key(len - 1, window, 0);
  const int* table = block_table + (long)span_of_token[t] * max_pages;
  const T* qrow = q + ((long)t * H + h) * row;
  for (int i = tid; i < row; i += kLatThreads) qs[i] = to_f32(qrow[i]);
  __syncthreads();
  float m = -INFINITY, l = 0.f;
  float acc[kLatMaxPer];
#pragma unroll
  for (int c = 0; c < kLatMaxPer; ++c) acc[c] = 0.f;
  for (int base = lo; base < len; base += kLatThreads) {
    const int key = base + tid;
    float s = -INFINITY;
    if (key < len) {
      const T* krow = cache + (long)table[key / page_size] * page_elems + (long)(key % page_size) * row;
      float dot = 0.f;
      for (int i = 0; i < row; ++i) dot = fmaf(qs[i], to_f32(krow[i]), dot);
      s = dot * scale;
    }
    const float m_new = fmaxf(m, block_max(s, red));
    const float alpha = expf(m - m_new);
    const float p = (s == -INFINITY) ? 0.f : expf(s - m_new);
    ps[tid] = p;
    l = l * alpha + block_sum(p, red);       // its barriers also publish ps
    m = m_new;
    const int nk = min(kLatThreads, len - base);
#pragma unroll
    for (int c = 0; c < kLatMaxPer; ++c) {
      const int e = tid + c * kLatThreads;
      acc[c] *= alpha;
      if (e < rank) {
        float a = acc[c];
        int pg = -1;
        const T* prow = nullptr;
        for (int k = 0; k < nk; ++k) {
          const int kk = base + k;
          if (kk / page_size != pg) {
            pg = kk / page_size;
            prow = cache + (long)table[pg] * page_elems;
          }
          a = fmaf(ps[k], to_f32(prow[(long)(kk % page_size) * row + e]), a);
        }
        acc[c] = a;
      }
    }
    __syncthreads();                         // ps is rewritten by the next round
  }
#pragma unroll
  for (int c = 0; c < kLatMaxPer; ++c) {
    const int e = tid + c * kLatThreads;
    if (e < rank) out[((long)t * H + h) * rank + e] = from_f32<T>(acc[c] / l);
  }
}

// attn_latent on the matrix cores (bfloat16).  A workgroup takes one token and up to 16 heads;
// its four waves take the token's keys in tiles of 32, round robin, and meet in LDS.  All heads
// read the same keys, so the 16 heads are the columns of one product:
// MFMA 16x16x32 (lane l: g = l/16, c = l%16): A[c][8g..8g+7], B[8g..8g+7][c], D[4g+i][c].
// Scores: A = 16 keys x 32 elements of their rows (one row per lane, straight from the page),
// B = the folded queries of the 16 heads, D[key 4g+i][head c].  Weighted sum: the 32 slots that
// are summed over are the keys (4g+j) of the tile's first half for j < 4 and of its second half for
// j >= 4, which is how a lane holds its probabilities; A = latents [element c][those keys], two
// 8-byte reads from the transposed copy.  NR: 16-element pieces of the latent a lane accumulates.
constexpr int kLatWaves = 4;

// KS: steps of 32 over a row whose pieces of the query a lane keeps in registers (0: it asks for
// them at every tile, for rows longer than the built sizes).
template <int NR, int KS>
__global__ __launch_bounds__(64 * kLatWaves) void attn_latent_mfma_kernel(
    const bf16_t* __restrict__ q, bf16_t* __restrict__ out, const bf16_t* __restrict__ cache,
    const int* __restrict__ positions, const int* __restrict__ span_of_token, const int* __restrict__ block_table,
    int max_pages, int page_size, unsigned page_magic, int H, int row, int rank, float scale, int window,
    float* __restrict__ part) {
  extern __shared__ float lat_red[];            // [kLatWaves][NR * 4 + 2][64]
  const int lane = threadIdx.x % kWave, wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
  const int g = lane / 16, c = lane % 16;
  const int t = blockIdx.x, h0 = blockIdx.y * 16;
  const int head = min(h0 + c, H - 1);
  const bool head_ok = h0 + c < H;
  const int len = positions[t] + 1;
  const int lo = first_key(len - 1, window, 0);        // the first key that is read
  const int* table = block_table + (long)span_of_token[t] * max_pages;
  const long page_elems = (long)page_size * (row + rank);
  const int ksteps = (row + 31) / 32, nr = rank / 16;
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  const bf16_t* qrow = q + ((long)t * H + head) * row;
  bf16x8 qreg[KS > 0 ? KS : 1];
#pragma unroll
  for (int kk = 0; kk < KS; ++kk) {
    const int d0 = 32 * kk + 8 * g;
    qreg[kk] = (d0 < row && head_ok) ? *reinterpret_cast<const bf16x8*>(qrow + d0) : zero8;
  }

  float m = -INFINITY, l = 0.f;
  floatx4 acc[NR];
#pragma unroll
  for (int r = 0; r < NR; ++r) acc[r] = floatx4{0.f, 0.f, 0.f, 0.f};

  // The tiles go in turn to the slices (workgroups of the same token and heads, blockIdx.z: where
  // tokens and heads alone leave CUs idle) and, within a slice, to the waves.
  const int nslices = gridDim.z, slice = blockIdx.z;
  const int tiles = (len + 31) / 32;
  const unsigned k_lane = c * row + 8 * g, v_lane = c * page_size + 4 * g;       // this lane's place in a half's rows and latents
  for (int tile = lo / 32 + slice * kLatWaves + wave; tile < tiles; tile += kLatWaves * nslices) {
    const int kb = tile * 32;
    // A half (16 keys) lies in one page (pages hold a multiple of 16 slots).  Loads carry no branch,
    // so that many are in flight: a half that is not read takes page 0, whose rows make scores that
    // are masked (a row is one key's alone) and whose latents are replaced by zeros.
    const bf16_t* pbase[2];
    int slot0[2];
    bool live[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int k0 = kb + 16 * u;
      live[u] = k0 < len && k0 + 16 > lo;                    // (a half behind the window may lie in a page that is gone)
      const int pi = live[u] ? (int)(__umulhi((unsigned)k0, page_magic) >> 3) : 0;   // k0 / page_size (see the launch)
      // (the same in every lane: said so explicitly, which keeps the addresses on the scalar unit)
      const int page = __builtin_amdgcn_readfirstlane(table[pi]);
      pbase[u] = cache + (long)(live[u] ? page : 0) * page_elems;
      slot0[u] = live[u] ? k0 - pi * page_size : 0;
    }
    const bf16_t* krow[2] = {pbase[0] + (long)slot0[0] * row, pbase[1] + (long)slot0[1] * row};      // + this lane's place
    const bf16_t* vt[2] = {pbase[0] + (long)page_size * row + slot0[0], pbase[1] + (long)page_size * row + slot0[1]};
    // ---- the latents' pieces, RB at a time: the first asked for behind the scores' products
    constexpr int RB = NR < 16 ? NR : 16;
    struct Piece {
      bf16x4 v[RB][2];
    };
    auto v_fetch = [&](int r0) -> Piece {
      Piece P;
#pragma unroll
      for (int r = 0; r < RB; ++r)
#pragma unroll
        for (int u = 0; u < 2; ++u)
          P.v[r][u] = *reinterpret_cast<const bf16x4*>(vt[u] + (long)(16 * min(r0 + r, nr - 1)) * page_size + v_lane);
      return P;
    };
    floatx4 s[2] = {floatx4{0.f, 0.f, 0.f, 0.f}, floatx4{0.f, 0.f, 0.f, 0.f}};
    if constexpr (KS > 0) {
      // the keys' pieces, KB steps at a time and one group ahead of the products
      constexpr int KB = KS % 6 == 0 ? 6 : KS % 5 == 0 ? 5 : 4;
      static_assert(KS % KB == 0, "whole groups of steps");
      bf16x8 a[2][KB][2];
      auto k_fetch = [&](bf16x8 (&dst)[KB][2], int j0) {
#pragma unroll
        for (int j = 0; j < KB; ++j)
#pragma unroll
          for (int u = 0; u < 2; ++u) {
            const int d0 = 32 * (j0 + j) + 8 * g;
            dst[j][u] = *reinterpret_cast<const bf16x8*>(krow[u] + k_lane + (unsigned)(d0 < row ? 32 * (j0 + j) : 0));
          }
      };
      k_fetch(a[0], 0);
#pragma unroll
      for (int j0 = 0; j0 < KS; j0 += KB) {
        if (j0 + KB < KS) k_fetch(a[(j0 / KB + 1) % 2], j0 + KB);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int j = 0; j < KB; ++j)
#pragma unroll
          for (int u = 0; u < 2; ++u) {
            const bool in = 32 * (j0 + j) + 8 * g < row;     // beyond a row: another slot's, anything
            s[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(in ? a[j0 / KB % 2][j][u] : zero8, qreg[j0 + j], s[u], 0, 0, 0);
          }
        __builtin_amdgcn_sched_barrier(0);
      }
    } else {
      for (int ks = 0; ks < ksteps; ++ks) {
        const int d0 = 32 * ks + 8 * g, da = d0 < row ? d0 : 0;
        const bf16x8 qv = *reinterpret_cast<const bf16x8*>(qrow + da);
        const bf16x8 qb = (d0 < row && head_ok) ? qv : zero8;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const bf16x8 a = *reinterpret_cast<const bf16x8*>(krow[u] + c * row + da);
          s[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(d0 < row ? a : zero8, qb, s[u], 0, 0, 0);
        }
      }
    }
    Piece piece = v_fetch(0);
    __builtin_amdgcn_sched_barrier(0);
    // ---- online softmax for this lane's head over its 8 keys, then over the 4 lanes of the column
    float tmax = -INFINITY;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = kb + 16 * u + 4 * g + i;
        s[u][i] = (key < len && key >= lo) ? s[u][i] * scale : -INFINITY;
        tmax = fmaxf(tmax, s[u][i]);
      }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, kWave));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, kWave));
    const float m_new = fmaxf(m, tmax);                    // finite: every tile holds a key that is read
    const float alpha = expf(m - m_new);
    bf16x8 pb;
    float psum = 0.f;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float p = (s[u][i] == -INFINITY) ? 0.f : expf(s[u][i] - m_new);
        const bf16_t pr = (bf16_t)p;
        pb[4 * u + i] = pr;
        psum += (float)pr;
      }
    l = l * alpha + psum;
    m = m_new;
    // ---- the weighted sum of the latents: slots beyond the last key may hold anything
    const bool edge = !live[0] || kb + 32 > len;
#pragma unroll
    for (int r = 0; r < NR; ++r) {
      if (r < nr) {
        acc[r] *= alpha;
        bf16x8 a;
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            a[4 * u + i] = (!edge || (live[u] && kb + 16 * u + 4 * g + i < len)) ? piece.v[r % RB][u][i] : (bf16_t)0.f;
        acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pb, acc[r], 0, 0, 0);
      }
      if (r % RB == RB - 1 && r + 1 < NR) {
        piece = v_fetch(r + 1);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
  }
  l += __shfl_xor(l, 16, kWave);
  l += __shfl_xor(l, 32, kWave);

  // ---- the waves meet: each leaves maximum, sum and output in LDS (lane-contiguous), then adds its share
  // of the elements of all of them in a fixed order with weights exp(m_w - max m) and writes
  constexpr int kRows = NR * 4 + 2;
  float* mine = lat_red + (long)wave * kRows * kWave + lane;
#pragma unroll
  for (int r = 0; r < NR; ++r)
#pragma unroll
    for (int i = 0; i < 4; ++i) mine[(4 * r + i) * kWave] = acc[r][i];
  mine[(NR * 4) * kWave] = m;
  mine[(NR * 4 + 1) * kWave] = l;
  __syncthreads();
  if (!head_ok) return;
  const float* all = lat_red + lane;
  float ww[kLatWaves], M = -INFINITY, L = 0.f;
#pragma unroll
  for (int w = 0; w < kLatWaves; ++w) M = fmaxf(M, all[(w * kRows + NR * 4) * kWave]);
#pragma unroll
  for (int w = 0; w < kLatWaves; ++w) {
    const float mw = all[(w * kRows + NR * 4) * kWave];
    ww[w] = (mw == -INFINITY) ? 0.f : expf(mw - M);        // (a slice beyond the token's keys has none)
    L += ww[w] * all[(w * kRows + NR * 4 + 1) * kWave];
  }
  // of a slice the sums as they are, with its maximum and its sum of probabilities: rows of rank + 2
  // floats; a slice without a key leaves a maximum of -inf and zeros
  float* prow = nslices > 1 ? part + (((long)t * H + head) * nslices + slice) * (rank + 2) : nullptr;
  const float inv = nslices > 1 ? 1.f : 1.f / L;
  bf16_t* orow = out + ((long)t * H + head) * rank;
#pragma unroll
  for (int j = 0; j < NR / kLatWaves; ++j) {
    const int r = wave * (NR / kLatWaves) + j;
    if (r >= nr) continue;
    floatx4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < kLatWaves; ++w)
#pragma unroll
      for (int i = 0; i < 4; ++i) o[i] = fmaf(ww[w], all[(w * kRows + 4 * r + i) * kWave], o[i]);
    if (nslices > 1) {                                       // (rows are 8-byte aligned)
      *reinterpret_cast<floatx2*>(prow + 16 * r + 4 * g) = floatx2{o[0], o[1]};
      *reinterpret_cast<floatx2*>(prow + 16 * r + 4 * g + 2) = floatx2{o[2], o[3]};
    } else {
      *reinterpret_cast<bf16x4*>(orow + 16 * r + 4 * g) =
          bf16x4{(bf16_t)(o[0] * inv), (bf16_t)(o[1] * inv), (bf16_t)(o[2] * inv), (bf16_t)(o[3] * inv)};
    }
  }
  if (nslices > 1 && wave == 0 && g == 0) *reinterpret_cast<floatx2*>(prow + rank) = floatx2{M, L};
}

// The same for steps of many tokens: a workgroup takes four consecutive tokens of the step and up
// to 16 heads, one token a wave.  Tokens of one request read the same keys: a tile of 32 keys
// (their rows, and their latents with the keys side by side) goes through LDS once for the
// four, which cuts the traffic between L2 and the CUs to a quarter.  Where the four tokens
// belong to several requests, the requests take their turns.  No merge: a wave has all keys
// of its token.  LDS: rows [32][row + 8], latents [rank][32 + 4] (padded against bank conflicts).
template <int NR, int KS>
__global__ __launch_bounds__(64 * kLatWaves) void attn_latent_block_kernel(
    const bf16_t* __restrict__ q, bf16_t* __restrict__ out, const bf16_t* __restrict__ cache,
    const int* __restrict__ positions, const int* __restrict__ span_of_token, const int* __restrict__ block_table,
    int max_pages, int page_size, unsigned page_magic, int n, int H, int row, int rank, float scale, int window, int redo) {
  extern __shared__ __attribute__((aligned(16))) bf16_t lat_tiles[];
  // page of a key without a division: page_magic = ceil(2^35 / page_size) from the host, exact for
  // keys below 2^24 and pages of up to 2,048 slots (checked at the launch)
  auto page_index = [&](int key) { return (int)(__umulhi((unsigned)key, page_magic) >> 3); };
  const int KLD = row + 8, VLD = 36;
  bf16_t* ks = lat_tiles;                      // [32][KLD]
  bf16_t* vs = lat_tiles + 32 * KLD;           // [rank][VLD]
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
  const int g = lane / 16, c = lane % 16;
  // later tokens of a prompt read more keys: the workgroups with the most to do start first
  const int t_first = (gridDim.x - 1 - blockIdx.x) * kLatWaves, h0 = blockIdx.y * 16;
  const int t = min(t_first + wave, n - 1);
  const bool token_ok = t_first + wave < n;
  const int head = min(h0 + c, H - 1);
  const bool head_ok = h0 + c < H;
  // behind attn_latent_columns_kernel: only where that left a column to be done
  if (redo && !__syncthreads_or(token_ok && head_ok && isnan((float)out[((long)t * H + head) * rank]))) return;
  const int my_span = span_of_token[t];
  const int len = positions[t] + 1;
  const int lo = first_key(len - 1, window, 0);
  const long page_elems = (long)page_size * (row + rank);
  const int ksteps = (row + 31) / 32, nr = rank / 16;
  const bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  const bf16_t* qrow = q + ((long)t * H + head) * row;
  const int rows_here = min(kLatWaves, n - t_first);
  bf16x8 qreg[KS > 0 ? KS : 1];
#pragma unroll
  for (int kk = 0; kk < KS; ++kk) {
    const int d0 = 32 * kk + 8 * g;
    qreg[kk] = (d0 < row && head_ok) ? *reinterpret_cast<const bf16x8*>(qrow + d0) : zero8;
  }

  float m = -INFINITY, l = 0.f;
  floatx4 acc[NR];
#pragma unroll
  for (int r = 0; r < NR; ++r) acc[r] = floatx4{0.f, 0.f, 0.f, 0.f};

  for (int first = 0; first < rows_here;) {
    const int span = span_of_token[t_first + first];
    int last = first;
    while (last + 1 < rows_here && span_of_token[t_first + last + 1] == span) ++last;
    const int group_len = positions[t_first + last] + 1;      // the group's last token reads the most keys
    const int group_lo = first_key(positions[t_first + first], window, 0);   // ... and its first the earliest (pages before it may be gone)
    const bool mine = token_ok && wave >= first && wave <= last;
    const int* table = block_table + (long)span * max_pages;
    // ---- a tile's way into LDS, 16 bytes at a time.  Thread tid moves pieces tid % 8, + 8, ... of key row
    // tid / 8, and 8 keys (part tid % 4) of elements tid / 4, + 64, ...: the same places in every tile.
    // For the built row sizes the pieces of the NEXT tile are asked for before the products of this
    // one and wait in registers meanwhile, their pages having been looked up a tile earlier, and no
    // load has a branch around it: a half (16 keys, in one page) that nobody reads takes page 0;
    // its scores are masked (a row is one key's alone), its latents replaced by zeros.
    constexpr int KP = KS > 0 ? KS / 2 : 1, VP = NR / 4;      // pieces a thread: of 32 rows of up to 32 KS, of 16 NR elements
    struct Stage {
      bf16x8 k[KP], v[VP];
    };
    struct Halves {
      int page[2];
    };
    const int row8 = row / 8;
    const int kr = tid / 8, kc = tid % 8, ve = tid / 4, vpart = tid % 4;
    auto half_live = [&](int k0) { return k0 < group_len && k0 + 16 > group_lo; };
    auto lookup = [&](int kb) -> Halves {
      Halves P;
#pragma unroll
      for (int u = 0; u < 2; ++u) P.page[u] = table[half_live(kb + 16 * u) ? page_index(kb + 16 * u) : 0];
      return P;
    };
    auto place = [&](const Halves& P, int k0, int u) -> const bf16_t* {      // the half's first row in its page
      const bool live = half_live(k0);
      return cache + (long)(live ? (u ? P.page[1] : P.page[0]) : 0) * page_elems;
    };
    auto slot_of = [&](int k0) { return half_live(k0) ? k0 - page_index(k0) * page_size : 0; };
    auto k_load = [&](const bf16_t* rows, int m) -> bf16x8 {
      const int piece = kc + 8 * m;
      return *reinterpret_cast<const bf16x8*>(rows + 8 * (piece < row8 ? piece : 0));
    };
    auto v_load = [&](const bf16_t* cols, int m) -> bf16x8 {
      return *reinterpret_cast<const bf16x8*>(cols + (long)min(ve + 64 * m, rank - 1) * page_size);
    };
    auto k_rows = [&](const Halves& P, int kb) {
      const int u = kr / 16, k0 = kb + 16 * u;
      return place(P, k0, u) + (long)(slot_of(k0) + kr % 16) * row;
    };
    auto v_cols = [&](const Halves& P, int kb) {
      const int u = vpart / 2, k0 = kb + 16 * u;
      return place(P, k0, u) + (long)page_size * row + slot_of(k0) + 8 * (vpart % 2);
    };
    auto k_store = [&](int m, const bf16x8& v) {
      const int piece = kc + 8 * m;
      if (piece < row8) *reinterpret_cast<bf16x8*>(ks + kr * KLD + 8 * piece) = v;
    };
    auto v_store = [&](int m, bf16x8 v, int kb) {
      if (ve + 64 * m >= rank) return;
      if (kb < group_lo || kb + 32 > group_len) {             // slots that may hold anything
        const int key = kb + 8 * vpart;
        const bool live = half_live(kb + 16 * (vpart / 2));
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = (live && key + j < group_len) ? v[j] : (bf16_t)0.f;
      }
      bf16_t* dst = vs + (ve + 64 * m) * VLD + 8 * vpart;     // 8-byte aligned
      *reinterpret_cast<bf16x4*>(dst) = bf16x4{v[0], v[1], v[2], v[3]};
      *reinterpret_cast<bf16x4*>(dst + 4) = bf16x4{v[4], v[5], v[6], v[7]};
    };
    auto fetch = [&](int kb, const Halves& P) -> Stage {
      Stage T;
      const bf16_t *kp = k_rows(P, kb), *vp = v_cols(P, kb);
#pragma unroll
      for (int m = 0; m < KP; ++m) T.k[m] = k_load(kp, m);
#pragma unroll
      for (int m = 0; m < VP; ++m) T.v[m] = v_load(vp, m);
      return T;
    };
    Stage st;
    Halves pages;
    const int kb0 = group_lo / 32 * 32;
    if constexpr (KS > 0) {
      pages = lookup(kb0);
      st = fetch(kb0, pages);
      pages = lookup(kb0 + 32);
    }
    for (int kb = kb0; kb < group_len; kb += 32) {
      __syncthreads();                                        // the tile before this one has been read
      if constexpr (KS > 0) {
#pragma unroll
        for (int m = 0; m < KP; ++m) k_store(m, st.k[m]);
#pragma unroll
        for (int m = 0; m < VP; ++m) v_store(m, st.v[m], kb);
      } else {
        pages = lookup(kb);
        const bf16_t *kp = k_rows(pages, kb), *vp = v_cols(pages, kb);
        for (int m = 0; 8 * m < row8; ++m) k_store(m, k_load(kp, m));
        for (int m = 0; 64 * m < rank; ++m) v_store(m, v_load(vp, m), kb);
      }
      __syncthreads();
      if constexpr (KS > 0) {                                 // (beyond the last tile: a valid address, dropped)
        st = fetch(kb + 32, pages);
        pages = lookup(kb + 64);
      }
      if (!mine || kb >= len || kb + 32 <= lo) continue;
      // ---- scores
      floatx4 s[2] = {floatx4{0.f, 0.f, 0.f, 0.f}, floatx4{0.f, 0.f, 0.f, 0.f}};
      auto score_step = [&](int kk, const bf16x8& qb) {
        const int d0 = 32 * kk + 8 * g;
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const bf16x8 a = d0 < row ? *reinterpret_cast<const bf16x8*>(ks + (16 * u + c) * KLD + d0) : zero8;
          s[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qb, s[u], 0, 0, 0);
        }
      };
      if constexpr (KS > 0) {
#pragma unroll
        for (int kk = 0; kk < KS; ++kk)
          if (kk < ksteps) score_step(kk, qreg[kk]);
      } else {
        for (int kk = 0; kk < ksteps; ++kk) {
          const int d0 = 32 * kk + 8 * g;
          score_step(kk, (d0 < row && head_ok) ? *reinterpret_cast<const bf16x8*>(qrow + d0) : zero8);
        }
      }
      float tmax = -INFINITY;
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = kb + 16 * u + 4 * g + i;
          s[u][i] = (key < len && key >= lo) ? s[u][i] * scale : -INFINITY;
          tmax = fmaxf(tmax, s[u][i]);
        }
      tmax = fmaxf(tmax, __shfl_xor(tmax, 16, kWave));
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, kWave));
      const float m_new = fmaxf(m, tmax);                    // finite: the tile holds a key of this token
      const float alpha = expf(m - m_new);
      bf16x8 pb;
      float psum = 0.f;
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float p = (s[u][i] == -INFINITY) ? 0.f : expf(s[u][i] - m_new);
          const bf16_t pr = (bf16_t)p;
          pb[4 * u + i] = pr;
          psum += (float)pr;
        }
      l = l * alpha + psum;
      m = m_new;
      // ---- the weighted sum of the latents (keys beyond this token's last: probability 0, and
      // what LDS holds of them is another token's key or zero, never anything else)
#pragma unroll
      for (int r = 0; r < NR; ++r) {
        if (r < nr) {
          acc[r] *= alpha;
          const bf16_t* vrow = vs + (16 * r + c) * VLD + 4 * g;
          const bf16x4 lo = *reinterpret_cast<const bf16x4*>(vrow);
          const bf16x4 hi = *reinterpret_cast<const bf16x4*>(vrow + 16);
          const bf16x8 a = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
          acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pb, acc[r], 0, 0, 0);
        }
      }
    }
    first = last + 1;
  }
  l += __shfl_xor(l, 16, kWave);
  l += __shfl_xor(l, 32, kWave);
  if (!token_ok || !head_ok) return;
  const float inv = 1.f / l;
  bf16_t* orow = out + ((long)t * H + head) * rank;
#pragma unroll
  for (int r = 0; r < NR; ++r) {
    if (r < nr) {
      bf16x4 v;
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = (bf16_t)(acc[r][i] * inv);
      *reinterpret_cast<bf16x4*>(orow + 16 * r + 4 * g) = v;
    }
  }
}

// The same for long steps of the common sizes (rank and rows in steps of 32): the (token, head) pairs of a
// step in a row are columns, 128 to a workgroup and 32 to a wave, and the products are MFMA 32x32x16
// (lane l: g = l/32, c = l%32: A[c][8g..8g+7], B[8g..8g+7][c], D[8(i/4) + 4g + i%4][c]).  Scores S^T =
// K Q^T: A = 32 keys x 16 of their rows from LDS, B = the columns' folded queries, which stay in
// registers; a lane holds 16 scores of one column, lane ^ 32 the other 16.  Weighted sum O^T += C^T P^T:
// the 16 slots of MFMA u are the keys 16u + 8(j/4) + 4g + j%4, j = 0..7, which are the scores 8u + j a
// lane holds; A = latents [element c][those keys], two 8-byte reads.
//
// A tile of 32 keys (rows, then latents with the keys side by side) goes from the pages straight into one of
// two LDS buffers (global loads that write LDS: 16 bytes a lane, a wave's 64 pieces in a row), the
// next tile's while this one is multiplied.  A wave cannot pad what it writes this way, so the 16-byte
// pieces of a row change places: piece p of key row k lies at p ^ (k & row_mask), piece p of
// element e's 32 keys at p ^ (e/4 % 4), which spreads a read over the banks.
//
// The accumulators fill the matrix unit's own registers, and the query's pieces most of the others: there
// is no room to bring an output to a new maximum.  Probabilities are taken relative to the largest score
// of the column's first tile instead, which is exact as long as no later score is more than kLatRange
// binary orders above it (32-bit and bfloat16 numbers have the same exponents, and what they hold relative to
// the largest is the same).  A column where one is leaves a NaN as its first element, and the launch
// behind this one (attn_latent_block_kernel, which otherwise ends at once) takes its place.
constexpr int kLatColumns = 128;      // of a workgroup
constexpr float kLatRange = 60.f;

__device__ __forceinline__ unsigned lds_address(const void* p) {
  return (unsigned)(size_t)(__attribute__((address_space(3))) const void*)p;
}
// 16 bytes a lane from base + offset (base, lds the same in every lane) to lds + 16 * lane.
__device__ __forceinline__ void load_to_lds(unsigned lds, const void* base, unsigned offset) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2" ::"s"(lds), "v"(offset), "s"(base) : "memory", "m0");
}
// The same from an address of the lane's own.
__device__ __forceinline__ void load_to_lds(unsigned lds, const void* address) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(lds), "v"(address) : "memory", "m0");
}

template <int NB, int KS>   // latents of 32 NB elements, rows of 16 KS
__global__ __launch_bounds__(64 * kLatWaves) __attribute__((amdgpu_waves_per_eu(NB <= 4 ? 2 : 1))) void attn_latent_columns_kernel(
    const bf16_t* __restrict__ q, bf16_t* __restrict__ out, const bf16_t* __restrict__ cache,
    const int* __restrict__ positions, const int* __restrict__ span_of_token, const int* __restrict__ block_table,
    int max_pages, int page_size, unsigned page_magic, int n, int H, float scale, int window) {
  constexpr int rank = 32 * NB, row = 16 * KS, row8 = row / 8;
  constexpr int row_mask = row8 % 8 == 0 ? 7 : row8 % 4 == 0 ? 3 : 1;
  extern __shared__ __attribute__((aligned(16))) bf16_t lat_tiles[];   // two buffers: [32][row], [rank][32]
  auto page_index = [&](int key) { return (int)(__umulhi((unsigned)key, page_magic) >> 3); };
  const int tid = threadIdx.x, lane = tid % kWave, wave = __builtin_amdgcn_readfirstlane(tid / kWave);
  const int g = lane / 32, c = lane % 32;
  constexpr int buf_elems = 32 * row + 32 * rank;
  // later tokens of a prompt read more keys: the workgroups with the most to do start first
  const long col0 = (long)(gridDim.x - 1 - blockIdx.x) * kLatColumns;
  const long ncols = (long)n * H;
  const int t_first = (int)(col0 / H), t_last = (int)((min(col0 + kLatColumns, ncols) - 1) / H);
  const long col = min(col0 + 32 * wave + c, ncols - 1);
  const bool col_ok = col0 + 32 * wave + c < ncols;
  const int t = (int)(col / H);
  const int my_span = span_of_token[t];
  const int len = positions[t] + 1;
  const int lo = first_key(len - 1, window, 0);
  const long page_elems = (long)page_size * (row + rank);
  const float c2 = scale * 1.4426950408889634f;             // scale * log2(e)
  bf16x8 qreg[KS];
#pragma unroll
  for (int kk = 0; kk < KS; ++kk) qreg[kk] = *reinterpret_cast<const bf16x8*>(q + col * row + 16 * kk + 8 * g);

  float m = -INFINITY, l = 0.f;
  floatx16 acc[NB];
#pragma unroll
  for (int r = 0; r < NB; ++r)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[r][i] = 0.f;

  // ---- where this lane's pieces of a tile come from.  Rows: load j of the wave (every fourth one) fills the
  // 64 pieces from 64 (4 j + wave) on; a half (16 keys, 2 row8 whole loads) lies in one page.  Latents:
  // load j fills 16 elements' pieces; the lane's piece, and with it its half, is the same in all of them.
  constexpr int KL = KS / 4 + (KS % 4 ? 1 : 0);              // loads of a wave: 32 rows of 2 KS pieces over 256 lanes
  unsigned k_off[KL];
#pragma unroll
  for (int j = 0; j < KL; ++j) {
    const int piece = 64 * (4 * j + wave) + lane;
    const int kr = piece / row8, kp = piece - kr * row8;
    k_off[j] = (unsigned)(((kr % 16) * row + 8 * (kp ^ (kr & row_mask))) * (int)sizeof(bf16_t));
  }
  const int v_piece = (lane % 4) ^ (lane / 16 % 4), v_half = v_piece / 2;
  const unsigned lds0 = lds_address(lat_tiles);
  // ... and where it reads them: four places each, the rest are constant distances
  int k_at[4], v_at[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    k_at[j] = c * row + 8 * ((2 * j + g) ^ (c & row_mask));
    v_at[j] = c * 32 + 8 * (j ^ (c / 4 % 4)) + 4 * g;
  }

  bool over = false;
  for (int first = t_first; first <= t_last;) {
    const int span = span_of_token[first];
    int last = first;
    while (last < t_last && span_of_token[last + 1] == span) ++last;
    const int group_len = positions[last] + 1;                // the span's last token here reads the most keys
    const int group_lo = first_key(positions[first], window, 0);   // ... and its first the earliest (pages before it may be gone)
    const bool mine = col_ok && my_span == span;
    const int* table = block_table + (long)span * max_pages;
    auto half_live = [&](int k0) { return k0 < group_len && k0 + 16 > group_lo; };
    struct Halves {
      int page[2];
    };
    // a vector load although the address is the same in every lane (see fetch: it has the loop's turn to arrive)
    auto lookup = [&](int kb) -> Halves {
      Halves P;
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        int index = half_live(kb + 16 * u) ? page_index(kb + 16 * u) : 0;
        asm volatile("" : "+v"(index));
        P.page[u] = table[index];
      }
      return P;
    };
    auto fetch = [&](int kb, const Halves& P, int buf) {
      const bf16_t* base[2];
      int slot[2];
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const int k0 = kb + 16 * u;
        const bool live = half_live(k0);                      // a half that nobody reads takes page 0
        const int page = __builtin_amdgcn_readfirstlane(P.page[u]);
        base[u] = cache + (long)(live ? page : 0) * page_elems;
        slot[u] = live ? k0 - page_index(k0) * page_size : 0;
      }
      const unsigned k_lds = lds0 + (unsigned)(buf * buf_elems) * (unsigned)sizeof(bf16_t);
      const unsigned v_lds = k_lds + (unsigned)(32 * row) * (unsigned)sizeof(bf16_t);
#pragma unroll
      for (int j = 0; j < KL; ++j) {
        const int load = 4 * j + wave;                        // of KS
        if (load >= KS) continue;
        const int u = 2 * load >= KS;                         // the first KS / 2 loads are the first half's
        load_to_lds(k_lds + 1024u * (unsigned)load, u ? base[1] + (long)slot[1] * row : base[0] + (long)slot[0] * row, k_off[j]);
      }
      const bf16_t* v0 = base[0] + (long)page_size * row + slot[0];
      const bf16_t* v1 = base[1] + (long)page_size * row + slot[1];
      const bf16_t* vsrc = (v_half ? v1 : v0) + 8 * (v_piece % 2) + (long)(lane / 4) * page_size;
#pragma unroll
      for (int j = 0; j < NB / 2; ++j) {
        const int load = 4 * j + wave;                        // of 2 NB
        load_to_lds(v_lds + 1024u * (unsigned)load, vsrc + (long)(16 * load) * page_size);
      }
    };
    const int kb0 = group_lo / 32 * 32;
    Halves pages = lookup(kb0);
    __syncthreads();                                          // the span before this one has been worked through
    fetch(kb0, pages, 0);
    pages = lookup(kb0 + 32);
    int buf = 0;
    for (int kb = kb0; kb < group_len; kb += 32, buf ^= 1) {
      asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");   // this wave's part of the tile is in LDS, its reads of the last one are done
      __builtin_amdgcn_s_barrier();
      asm volatile("" ::: "memory");
      if (kb + 32 < group_len) {                              // (the same for all)
        fetch(kb + 32, pages, buf ^ 1);
        pages = lookup(kb + 64);
      }
      bf16_t* const ks = lat_tiles + buf * buf_elems;         // [32][row]
      bf16_t* const vs = ks + 32 * row;                       // [rank][32]
      if (kb + 32 > group_len || !half_live(kb)) {            // latents of slots that may hold anything become zeros
        for (int i = tid; i < 32 * rank; i += 64 * kLatWaves) {
          const int key = kb + i % 32;
          if (key >= group_len || !half_live(kb + i % 32 / 16 * 16)) {
            const int e = i / 32, piece = i % 32 / 8;
            vs[e * 32 + 8 * (piece ^ (e / 4 % 4)) + i % 8] = (bf16_t)0.f;
          }
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        asm volatile("" ::: "memory");
      }
      if (!__any(mine && kb < len && kb + 32 > lo)) continue;
      // ---- scores: this lane's key row is c
      // (a group of pieces is read while the one before it is multiplied, and no more: registers)
      constexpr int kGroup = 2;
      floatx16 s0 = {}, s1 = {};
      bf16x8 ka[2][kGroup];
#pragma unroll
      for (int j = 0; j < kGroup; ++j) ka[0][j] = *reinterpret_cast<const bf16x8*>(ks + k_at[j]);
#pragma unroll
      for (int k0 = 0; k0 < KS; k0 += kGroup) {               // piece 2 kk + g of the row, at its swapped place
#pragma unroll
        for (int j = 0; j < kGroup; ++j) {
          const int kk = k0 + kGroup + j;
          if (kk < KS) ka[(k0 / kGroup + 1) % 2][j] = *reinterpret_cast<const bf16x8*>(ks + k_at[kk % 4] + 64 * (kk / 4));
        }
        __builtin_amdgcn_sched_barrier(0);
        s0 = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ka[k0 / kGroup % 2][0], qreg[k0], s0, 0, 0, 0);
        s1 = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ka[k0 / kGroup % 2][1], qreg[k0 + 1], s1, 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0);
      }
      const int hi_e = mine ? len - 1 - kb - 4 * g : -1, lo_e = lo - kb - 4 * g;    // offsets that this lane's column reads
      float tmax = -INFINITY;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int e = 8 * (i / 4) + i % 4;
        s0[i] = (e <= hi_e && e >= lo_e) ? (s0[i] + s1[i]) * c2 : -INFINITY;
        tmax = fmaxf(tmax, s0[i]);
      }
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, kWave));
      if (m == -INFINITY) m = tmax;                           // the column's first keys
      over |= tmax > m + kLatRange;
      const float mref = m == -INFINITY ? 0.f : m;            // (a column without a key so far: every score is -inf)
      bf16x8 pb[2];
      float psum = 0.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const bf16_t p = (bf16_t)__builtin_amdgcn_exp2f(s0[i] - mref);      // exp2(-inf) = 0
        pb[i / 8][i % 8] = p;
        psum += (float)p;
      }
      l += psum;
      // ---- the weighted sum of the latents
      {
        bf16x4 va[2][4];
#pragma unroll
        for (int j = 0; j < 4; ++j) va[0][j] = *reinterpret_cast<const bf16x4*>(vs + v_at[j]);
#pragma unroll
        for (int r = 0; r < NB; ++r) {
          if (r + 1 < NB)
#pragma unroll
            for (int j = 0; j < 4; ++j) va[(r + 1) % 2][j] = *reinterpret_cast<const bf16x4*>(vs + v_at[j] + 1024 * (r + 1));
          __builtin_amdgcn_sched_barrier(0);
#pragma unroll
          for (int u = 0; u < 2; ++u) {
            const bf16x4 a0 = va[r % 2][2 * u], a1 = va[r % 2][2 * u + 1];
            const bf16x8 a = {a0[0], a0[1], a0[2], a0[3], a1[0], a1[1], a1[2], a1[3]};
            acc[r] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, pb[u], acc[r], 0, 0, 0);
          }
          __builtin_amdgcn_sched_barrier(0);
        }
      }
    }
    first = last + 1;
  }
  l += __shfl_xor(l, 32, kWave);
  if (!col_ok) return;
  const float inv = over ? NAN : 1.f / l;
  bf16_t* orow = out + col * rank;
#pragma unroll
  for (int r = 0; r < NB; ++r)
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      bf16x4 v;
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = (bf16_t)(acc[r][4 * b + i] * inv);
      *reinterpret_cast<bf16x4*>(orow + 32 * r + 8 * b + 4 * g) = v;
    }
}

template <int NB, int KS>
static int launch_latent_columns(const void* q, void* out, const void* cache, const int* positions, const int* span_of_token,
                                 const int* block_table, int max_pages, int page_size, int n, int H, float scale, int window,
                                 hipStream_t stream) {
  const size_t lds = 2 * (size_t)(32 * 16 * KS + 32 * 32 * NB) * sizeof(bf16_t);
  static size_t raised_to = 64 * 1024;
  if (lds > raised_to) {
    hipError_t e = hipFuncSetAttribute((const void*)attn_latent_columns_kernel<NB, KS>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) KLLM_FAIL((int)e, "attn_latent: cannot raise the LDS limit: %s", hipGetErrorString(e));
    raised_to = lds;
  }
  const unsigned page_magic = (unsigned)(((1ull << 35) + page_size - 1) / page_size);
  hipLaunchKernelGGL((attn_latent_columns_kernel<NB, KS>), dim3(ceil_div((long)n * H, kLatColumns)), dim3(64 * kLatWaves), lds, stream,
                     (const bf16_t*)q, (bf16_t*)out, (const bf16_t*)cache, positions, span_of_token, block_table, max_pages,
                     page_size, page_magic, n, H, scale, window);
  return 0;
}

// The slices' results of one (token, head) become its output: weights exp(m_s - max m).  A lane takes one
// slice's maximum and sum (up to 64 slices) and works out its weight; the weights wait in LDS while
// eight slices' outputs at a time are asked for.
__global__ __launch_bounds__(kLatThreads) void attn_latent_merge_kernel(const float* __restrict__ part,
                                                                        bf16_t* __restrict__ out, int rank, int nslices) {
  __shared__ float weight[kWave];
  const long th = blockIdx.x;
  const long stride = rank + 2;
  const float* rows = part + th * nslices * stride;
  const int lane = threadIdx.x % kWave;
  const bool there = lane < nslices;
  const float ms = there ? rows[lane * stride + rank] : -INFINITY;
  const float ls = there ? rows[lane * stride + rank + 1] : 0.f;
  const float M = wave_max(ms);                               // finite: some slice holds the token's own key
  const float w = ms == -INFINITY ? 0.f : expf(ms - M);
  const float inv = 1.f / wave_sum(w * ls);
  if (threadIdx.x < kWave) weight[lane] = w * inv;            // 0 for a slice without a key
  __syncthreads();
  for (int e = threadIdx.x; e < rank; e += kLatThreads) {
    float o = 0.f;
    for (int s0 = 0; s0 < nslices; s0 += 8) {
      float v[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = rows[min(s0 + j, nslices - 1) * stride + e];
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (s0 + j < nslices && weight[s0 + j] != 0.f) o = fmaf(weight[s0 + j], v[j], o);
    }
    out[th * rank + e] = (bf16_t)o;
  }
}

template <int NR, int KS>
static void launch_latent_mfma(const void* q, void* out, const void* cache, const int* positions, const int* span_of_token,
                               const int* block_table, int max_pages, int page_size, int n, int H, int row, int rank,
                               float scale, int window, float* part, int nslices, int redo, hipStream_t stream) {
  const size_t lds = (size_t)kLatWaves * (NR * 4 + 2) * kWave * sizeof(float);
  const unsigned page_magic = (unsigned)(((1ull << 35) + page_size - 1) / page_size);
  static int raised = 0;
  if (lds > 64 * 1024 && !raised) {
    (void)hipFuncSetAttribute((const void*)attn_latent_mfma_kernel<NR, KS>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    raised = 1;
  }
  if (nslices == 0) {       // steps of many tokens: four tokens a workgroup, their keys through LDS
    const size_t tiles = ((size_t)32 * (row + 8) + (size_t)rank * 36) * sizeof(bf16_t);
    static size_t raised_to = 64 * 1024;
    if (tiles > raised_to) {
      (void)hipFuncSetAttribute((const void*)attn_latent_block_kernel<NR, KS>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)tiles);
      raised_to = tiles;
    }
    hipLaunchKernelGGL((attn_latent_block_kernel<NR, KS>), dim3((n + kLatWaves - 1) / kLatWaves, (H + 15) / 16), dim3(64 * kLatWaves),
                       tiles, stream, (const bf16_t*)q, (bf16_t*)out, (const bf16_t*)cache, positions, span_of_token,
                       block_table, max_pages, page_size, page_magic, n, H, row, rank, scale, window, redo);
    return;
  }
  hipLaunchKernelGGL((attn_latent_mfma_kernel<NR, KS>), dim3(n, (H + 15) / 16, nslices), dim3(64 * kLatWaves), lds, stream,
                     (const bf16_t*)q, (bf16_t*)out, (const bf16_t*)cache, positions, span_of_token, block_table, max_pages,
                     page_size, page_magic, H, row, rank, scale, window, part);
  if (nslices > 1)
    hipLaunchKernelGGL(attn_latent_merge_kernel, dim3(n * H), dim3(kLatThreads), 0, stream, part, (bf16_t*)out, rank, nslices);
}

// attended: [n][H][rank]; w_uv [H * dv][rank]; gate: [nsplit][n][H * dv] sums ([H] with by_head) or null.
template <typename T>
__global__ __launch_bounds__(kLatThreads) void latent_out_kernel(
    const T* __restrict__ attended, const T* __restrict__ w_uv, const float* __restrict__ gate, int nsplit,
    long split_stride, long gate_stride, int by_head, T* __restrict__ out, int H, int dv, int rank) {
  extern __shared__ float al[];          // [rank]
  const long t = blockIdx.x;
  const int h = blockIdx.y, tid = threadIdx.x;
  const T* src = attended + (t * H + h) * rank;
  for (int i = tid; i < rank; i += kLatThreads) al[i] = to_f32(src[i]);
  __syncthreads();
  for (int j = tid; j < dv; j += kLatThreads) {
    const T* w = w_uv + ((long)h * dv + j) * rank;
    float acc = 0.f;
    for (int r = 0; r < rank; ++r) acc = fmaf(al[r], to_f32(w[r]), acc);
    const long col = (long)h * dv + j;
    if (gate) {
      float g = 0.f;
      for (int s = 0; s < nsplit; ++s) g += gate[s * split_stride + t * gate_stride + (by_head ? h : col)];
      acc *= sigmoid_f32(g);
    }
    out[t * H * dv + col] = from_f32<T>(acc);
  }
}

// The two products with a head's own matrix on the matrix cores (bfloat16), MFMA 16x16x32 as
// above: a wave takes 16 outputs (rows of the head's matrix, one per lane, 16 bytes at a time)
// and 16 tokens, a workgroup four such pieces of 16 outputs.
//   latent_out:   out[t][h][j] = sum_r W_uv[h dv + j][r] attended[t][h][r], times the gate
//   latent_query: out[t][h][r] = sum_i W_ukT[h][r][i] q[t][h][i] (W_ukT: the head's matrix
//                 transposed once, when the weights are bound), and the rotated part beside it
__global__ __launch_bounds__(kLatThreads) void latent_out_mfma_kernel(
    const bf16_t* __restrict__ attended, const bf16_t* __restrict__ w_uv, const float* __restrict__ gate, int nsplit,
    long split_stride, long gate_stride, int by_head, bf16_t* __restrict__ out, int n, int H, int dv, int rank) {
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int g = lane / 16, c = lane % 16;
  const int h = blockIdx.y;
  const int j0 = (blockIdx.z * 4 + wave) * 16;
  if (j0 >= dv) return;
  const int t = min((int)blockIdx.x * 16 + c, n - 1);
  const int j = min(j0 + c, dv - 1);
  const bf16_t* wrow = w_uv + ((long)h * dv + j) * rank;
  const bf16_t* arow = attended + ((long)t * H + h) * rank;
  floatx4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 8 * g; k0 < rank; k0 += 32) {            // rank % 32 == 0 (the launch): every lane takes every step
    const bf16x8 a = *reinterpret_cast<const bf16x8*>(wrow + k0);
    const bf16x8 b = *reinterpret_cast<const bf16x8*>(arow + k0);
    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc, 0, 0, 0);
  }
  const int tt = blockIdx.x * 16 + c;
  if (tt >= n) return;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int jj = j0 + 4 * g + i;
    if (jj >= dv) continue;
    const long col = (long)h * dv + jj;
    float v = acc[i];
    if (gate) {
      float gs = 0.f;
      for (int s = 0; s < nsplit; ++s) gs += gate[s * split_stride + tt * gate_stride + (by_head ? h : col)];
      v *= sigmoid_f32(gs);
    }
    out[(long)tt * H * dv + col] = (bf16_t)v;
  }
}

__global__ __launch_bounds__(kLatThreads) void latent_query_mfma_kernel(
    const float* __restrict__ q, int nsplit, long split_stride, const bf16_t* __restrict__ w_ukt,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, bf16_t* __restrict__ out, int n, int H, int d,
    int dr, int rank) {
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int g = lane / 16, c = lane % 16;
  const int h = blockIdx.y;
  const int hw = d + dr, half = dr / 2;
  const int t = min((int)blockIdx.x * 16 + c, n - 1);
  const int tt = blockIdx.x * 16 + c;
  const float* in = q + ((long)t * H + h) * hw;
  const int r0 = (blockIdx.z * 4 + wave) * 16;
  if (r0 < rank) {
    const int r = min(r0 + c, rank - 1);
    const bf16_t* wrow = w_ukt + ((long)h * rank + r) * d;
    floatx4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 8 * g; k0 < d; k0 += 32) {               // d % 32 == 0 (the launch)
      const bf16x8 a = *reinterpret_cast<const bf16x8*>(wrow + k0);
      bf16x8 b;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        float v = 0.f;
        for (int s = 0; s < nsplit; ++s) v += in[s * split_stride + k0 + e];
        b[e] = (bf16_t)v;
      }
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc, 0, 0, 0);
    }
    if (tt < n) {
      bf16_t* dst = out + ((long)tt * H + h) * (rank + dr);
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (r0 + 4 * g + i < rank) dst[r0 + 4 * g + i] = (bf16_t)acc[i];
    }
  }
  // the rotated part: the workgroup's first piece of outputs takes it along
  if (blockIdx.z == 0 && wave == 0 && tt < n) {
    bf16_t* dst = out + ((long)tt * H + h) * (rank + dr);
    for (int i = g; i < half; i += 4) {
      float a = 0.f, b = 0.f;
      for (int s = 0; s < nsplit; ++s) {
        a += in[s * split_stride + d + i];
        b += in[s * split_stride + d + half + i];
      }
      const float cs = cos_t[(long)tt * half + i], sn = sin_t[(long)tt * half + i];
      dst[rank + i] = (bf16_t)(a * cs - b * sn);
      dst[rank + half + i] = (bf16_t)(b * cs + a * sn);
    }
  }
}

// The same two products for steps of many tokens, MFMA 32x32x16 (lane l: g = l/32, c = l%32: A[c][8g..],
// B[8g..][c], D[8(i/4) + 4g + i%4][c]): a workgroup takes 64 tokens of a head, A = 32 outputs (rows of the
// head's matrix), B = 32 tokens; a lane then holds pieces of four neighbouring outputs of one token.
constexpr int kLatTokens = 64;

// DS = d / 16.  The tokens' queries (their slices added, in the compute type) pass through LDS once
// for all outputs; a wave takes every fourth piece of 32 outputs.
template <int DS>
__global__ __launch_bounds__(kLatThreads) void latent_query_block_kernel(
    const float* __restrict__ q, int nsplit, long split_stride, const bf16_t* __restrict__ w_ukt,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, bf16_t* __restrict__ out, int n, int H, int dr,
    int rank) {
  constexpr int d = 16 * DS, LD = d + 8;
  __shared__ __attribute__((aligned(16))) bf16_t qs[kLatTokens * LD];
  const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
  const int g = lane / 32, c = lane % 32;
  const int h = blockIdx.x, t0 = blockIdx.y * kLatTokens;
  const int hw = d + dr, half = dr / 2;
  const long row_out = (long)H * (rank + dr);
  for (int i = tid; i < kLatTokens * (d / 4); i += kLatThreads) {
    const int tt = i / (d / 4), e = 4 * (i % (d / 4));
    const float* in = q + ((long)min(t0 + tt, n - 1) * H + h) * hw + e;
    float v[4] = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < nsplit; ++s)
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] += in[s * split_stride + j];
    *reinterpret_cast<bf16x4*>(qs + tt * LD + e) = bf16x4{(bf16_t)v[0], (bf16_t)v[1], (bf16_t)v[2], (bf16_t)v[3]};
  }
  // the rotated part beside it
  for (int i = tid; i < kLatTokens * half; i += kLatThreads) {
    const int tt = i / half, e = i % half, t = t0 + tt;
    if (t >= n) break;
    const float* in = q + ((long)t * H + h) * hw + d + e;
    float a = 0.f, b = 0.f;
    for (int s = 0; s < nsplit; ++s) {
      a += in[s * split_stride];
      b += in[s * split_stride + half];
    }
    const float cs = cos_t[(long)t * half + e], sn = sin_t[(long)t * half + e];
    bf16_t* dst = out + t * row_out + (long)h * (rank + dr) + rank + e;
    dst[0] = (bf16_t)(a * cs - b * sn);
    dst[half] = (bf16_t)(b * cs + a * sn);
  }
  __syncthreads();
  for (int r0 = 32 * wave; r0 < rank; r0 += 32 * (kLatThreads / kWave)) {
    const bf16_t* wrow = w_ukt + ((long)h * rank + min(r0 + c, rank - 1)) * d + 8 * g;
    bf16x8 a[DS];
#pragma unroll
    for (int k = 0; k < DS; ++k) a[k] = *reinterpret_cast<const bf16x8*>(wrow + 16 * k);
#pragma unroll
    for (int tb = 0; tb < kLatTokens / 32; ++tb) {
      floatx16 acc = {};
#pragma unroll
      for (int k = 0; k < DS; ++k)
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[k], *reinterpret_cast<const bf16x8*>(qs + (32 * tb + c) * LD + 16 * k + 8 * g),
                                                      acc, 0, 0, 0);
      const int t = t0 + 32 * tb + c;
      if (t >= n) continue;
      bf16_t* dst = out + t * row_out + (long)h * (rank + dr) + r0 + 4 * g;
#pragma unroll
      for (int b = 0; b < 4; ++b)
        if (r0 + 8 * b + 4 * g < rank)                        // rank in steps of 4 (the launch)
          *reinterpret_cast<bf16x4*>(dst + 8 * b) =
              bf16x4{(bf16_t)acc[4 * b], (bf16_t)acc[4 * b + 1], (bf16_t)acc[4 * b + 2], (bf16_t)acc[4 * b + 3]};
    }
  }
}

// A wave takes 32 outputs and 32 of the tokens, the rank in steps of 16, eight steps' pieces in flight.
__global__ __launch_bounds__(kLatThreads) void latent_out_block_kernel(
    const bf16_t* __restrict__ attended, const bf16_t* __restrict__ w_uv, const float* __restrict__ gate, int nsplit,
    long split_stride, long gate_stride, int by_head, bf16_t* __restrict__ out, int n, int H, int dv, int rank) {
  constexpr int kAhead = 8;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int g = lane / 32, c = lane % 32;
  const int h = blockIdx.x, t0 = blockIdx.y * kLatTokens + 32 * (wave % 2);
  const int j0 = (2 * blockIdx.z + wave / 2) * 32;
  if (j0 >= dv || t0 >= n) return;
  const bf16_t* wrow = w_uv + ((long)h * dv + min(j0 + c, dv - 1)) * rank + 8 * g;
  const bf16_t* arow = attended + ((long)min(t0 + c, n - 1) * H + h) * rank + 8 * g;
  floatx16 acc = {};
  const int steps = rank / 16;
  for (int k0 = 0; k0 < steps; k0 += kAhead) {
    bf16x8 a[kAhead], b[kAhead];
#pragma unroll
    for (int k = 0; k < kAhead; ++k) {
      const int at = 16 * min(k0 + k, steps - 1);
      a[k] = *reinterpret_cast<const bf16x8*>(wrow + at);
      b[k] = *reinterpret_cast<const bf16x8*>(arow + at);
    }
#pragma unroll
    for (int k = 0; k < kAhead; ++k)
      if (k0 + k < steps) acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[k], b[k], acc, 0, 0, 0);
  }
  const int t = t0 + c;
  if (t >= n) return;
#pragma unroll
  for (int b = 0; b < 4; ++b) {
    const int j = j0 + 8 * b + 4 * g;
    if (j >= dv) continue;                                    // dv in steps of 4 (the launch)
    float z[4] = {0.f, 0.f, 0.f, 0.f};
    if (gate) {
      const float* at = gate + t * gate_stride + (by_head ? h : (long)h * dv + j);
      for (int s = 0; s < nsplit; ++s)
#pragma unroll
        for (int e = 0; e < 4; ++e) z[e] += at[s * split_stride + (by_head ? 0 : e)];
    }
    bf16x4 v;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = (bf16_t)(gate ? acc[4 * b + e] * sigmoid_f32(z[e]) : acc[4 * b + e]);
    *reinterpret_cast<bf16x4*>(out + ((long)t * H + h) * dv + j) = v;
  }
}

}  // namespace kllm

using namespace kllm;

extern "C" int kllm_latent_max_row(void) { return kLatMaxRow; }

extern "C" int kllm_latent_kv_append(const float* dkv, int nsplit, long split_stride, const float* weight, float eps,
                                     const float* cos_t, const float* sin_t, void* cache, const int* positions,
                                     const int* span_of_token, const int* block_table, int max_pages, int page_size,
                                     int n, int rank, int dr, int dtype, long in_stride, hipStream_t stream) {
  KLLM_REQUIRE(dkv && weight && cos_t && sin_t && cache && positions && span_of_token && block_table,
               "latent_kv_append: null pointer");
  KLLM_REQUIRE(n > 0 && nsplit >= 1 && rank > 0 && dr > 0 && dr % 2 == 0 && rank + dr <= kLatMaxRow,
               "latent_kv_append: bad sizes n=%d rank=%d dr=%d (rows of up to %d)", n, rank, dr, kLatMaxRow);
  KLLM_REQUIRE(max_pages > 0 && page_size > 0, "latent_kv_append: bad cache sizes");
  KLLM_REQUIRE(dtype == DT_F32 || dtype == DT_BF16, "latent_kv_append: unknown dtype %d", dtype);
  if (dtype == DT_F32)
    hipLaunchKernelGGL(latent_kv_append_kernel<float>, dim3(n), dim3(kLatThreads), 0, stream, dkv, nsplit, split_stride,
                       weight, eps, cos_t, sin_t, (float*)cache, positions, span_of_token, block_table, max_pages,
                       page_size, rank, dr, in_stride);
  else
    hipLaunchKernelGGL(latent_kv_append_kernel<bf16_t>, dim3(n), dim3(kLatThreads), 0, stream, dkv, nsplit,
                       split_stride, weight, eps, cos_t, sin_t, (bf16_t*)cache, positions, span_of_token, block_table,
                       max_pages, page_size, rank, dr, in_stride);
  KLLM_CHECK_LAUNCH("latent_kv_append");
  return 0;
}

extern "C" int kllm_latent_norm(const float* in, int nsplit, long split_stride, long in_stride, const float* weight,
                                float eps, void* out, int n, int r, int dtype, hipStream_t stream) {
  KLLM_REQUIRE(in && weight && out && n > 0 && r > 0 && nsplit >= 1 && in_stride >= r, "latent_norm: null pointer or bad sizes");
  KLLM_REQUIRE(dtype == DT_F32 || dtype == DT_BF16, "latent_norm: unknown dtype %d", dtype);
#define KLLM_LN(T, PER)                                                                                              \
  hipLaunchKernelGGL((latent_norm_kernel<T, PER>), dim3(n), dim3(kLatThreads), 0, stream, in, nsplit, split_stride,  \
                     in_stride, weight, eps, (T*)out, r)
#define KLLM_LNS(T)                                                        \
  do {                                                                     \
    if (r <= 4 * kLatThreads) KLLM_LN(T, 4);                               \
    else if (r <= 16 * kLatThreads) KLLM_LN(T, 16);                        \
    else KLLM_LN(T, 0);                                                    \
  } while (0)
  if (dtype == DT_F32) KLLM_LNS(float); else KLLM_LNS(bf16_t);
#undef KLLM_LNS
#undef KLLM_LN
  KLLM_CHECK_LAUNCH("latent_norm");
  return 0;
}

extern "C" int kllm_latent_query(const float* q, int nsplit, long split_stride, const void* w_uk, const float* cos_t,
                                 const float* sin_t, void* out, int n, int H, int d, int dr, int rank, int dtype,
                                 int transposed, hipStream_t stream) {
  KLLM_REQUIRE(q && w_uk && cos_t && sin_t && out, "latent_query: null pointer");
  KLLM_REQUIRE(n > 0 && nsplit >= 1 && H > 0 && H <= 65535 && d > 0 && dr > 0 && dr % 2 == 0 && rank > 0 &&
                   rank + dr <= kLatMaxRow && d + dr <= 4096,
               "latent_query: bad sizes n=%d H=%d d=%d dr=%d rank=%d", n, H, d, dr, rank);
  KLLM_REQUIRE(dtype == DT_F32 || dtype == DT_BF16, "latent_query: unknown dtype %d", dtype);
  if (transposed) {     // w_uk is [H][rank][d]: the kernel on the matrix cores
    KLLM_REQUIRE(dtype == DT_BF16 && d % 32 == 0 && ((uintptr_t)w_uk & 15) == 0,
                 "latent_query: the transposed matrix goes with bfloat16 and head sizes in steps of 32 (d=%d)", d);
    if (n >= kLatTokens && rank % 4 == 0 && dr % 4 == 0 && d <= 256 && ((uintptr_t)out & 7) == 0 && (n + kLatTokens - 1) / kLatTokens <= 65535) {
      const dim3 grid(H, (n + kLatTokens - 1) / kLatTokens);
#define KLLM_LQ(DS)                                                                                                   \
  case DS / 2:                                                                                                        \
    hipLaunchKernelGGL(latent_query_block_kernel<DS>, grid, dim3(kLatThreads), 0, stream, q, nsplit, split_stride,    \
                       (const bf16_t*)w_uk, cos_t, sin_t, (bf16_t*)out, n, H, dr, rank);                              \
    break
      switch (d / 32) { KLLM_LQ(2); KLLM_LQ(4); KLLM_LQ(6); KLLM_LQ(8); KLLM_LQ(10); KLLM_LQ(12); KLLM_LQ(14); KLLM_LQ(16); }
#undef KLLM_LQ
      KLLM_CHECK_LAUNCH("latent_query");
      return 0;
    }
    hipLaunchKernelGGL(latent_query_mfma_kernel, dim3((n + 15) / 16, H, (rank + 63) / 64), dim3(kLatThreads), 0, stream, q,
                       nsplit, split_stride, (const bf16_t*)w_uk, cos_t, sin_t, (bf16_t*)out, n, H, d, dr, rank);
    KLLM_CHECK_LAUNCH("latent_query");
    return 0;
  }
  const size_t lds = (size_t)(d + dr) * sizeof(float);
  if (dtype == DT_F32)
    hipLaunchKernelGGL(latent_query_kernel<float>, dim3(n, H), dim3(kLatThreads), lds, stream, q, nsplit, split_stride,
                       (const float*)w_uk, cos_t, sin_t, (float*)out, H, d, dr, rank);
  else
    hipLaunchKernelGGL(latent_query_kernel<bf16_t>, dim3(n, H), dim3(kLatThreads), lds, stream, q, nsplit, split_stride,
                       (const bf16_t*)w_uk, cos_t, sin_t, (bf16_t*)out, H, d, dr, rank);
  KLLM_CHECK_LAUNCH("latent_query");
  return 0;
}

extern "C" int kllm_attn_latent(const void* q, void* out, const void* cache, const int* positions,
                                const int* span_of_token, const int* block_table, int max_pages, int page_size, int n,
                                int H, int row, int rank, float scale, int dtype, int mode, float* part, long part_floats, int nslices,
                                int window, hipStream_t stream) {
  KLLM_REQUIRE(q && out && cache && positions && span_of_token && block_table, "attn_latent: null pointer");
  KLLM_REQUIRE(n > 0 && H > 0 && H <= 65535 && rank > 0 && rank <= row && row <= kLatMaxRow,
               "attn_latent: bad sizes n=%d H=%d row=%d rank=%d (rows of up to %d)", n, H, row, rank, kLatMaxRow);
  KLLM_REQUIRE(max_pages > 0 && page_size > 0 && window >= 0, "attn_latent: bad cache sizes or window");
  KLLM_REQUIRE(dtype == DT_F32 || dtype == DT_BF16, "attn_latent: unknown dtype %d", dtype);
  if (dtype == DT_BF16 && mode != 1 && rank % 16 == 0 && row % 8 == 0 && rank <= 512 && page_size % 16 == 0 &&
      page_size <= 2048 && (long)max_pages * page_size <= (1L << 24) &&
      ((uintptr_t)q & 15) == 0 && ((uintptr_t)cache & 15) == 0 && ((uintptr_t)out & 7) == 0) {
    KLLM_REQUIRE(nslices >= 0 && nslices <= 64 && (nslices <= 1 || (part && ((uintptr_t)part & 7) == 0 && part_floats >= (long)n * H * nslices * (rank + 2))),
                 "attn_latent: %d slices need room for %d tokens x %d heads x %d slices x (%d + 2) floats", nslices, n, H,
                 nslices, rank);
    int redo = 0;
    if (nslices == 0 && (long)n * H / kLatColumns < (1L << 30)) {
      // the sizes that are built for long steps: (rank, row) = 32 NB, 16 KS
#define KLLM_LATC(NB, KS)                                                                                               \
  if (rank == 32 * NB && row == 16 * KS) {                                                                              \
    if (int rc = launch_latent_columns<NB, KS>(q, out, cache, positions, span_of_token, block_table, max_pages, page_size, n, \
                                               H, scale, window, stream))                                               \
      return rc;                                                                                                        \
    redo = 1;                                                                                                           \
  }
      KLLM_LATC(2, 6) KLLM_LATC(2, 8) KLLM_LATC(4, 10) KLLM_LATC(4, 12) KLLM_LATC(8, 18) KLLM_LATC(8, 20) KLLM_LATC(16, 34)
      KLLM_LATC(16, 36)
#undef KLLM_LATC
    }
    // the latent's accumulators and the query's pieces in registers: built for ranks up to 128, 256 and
    // 512 with rows of up to 256, 384 and 640; longer rows ask for the query at every tile
#define KLLM_LAT(NR, KS) launch_latent_mfma<NR, KS>(q, out, cache, positions, span_of_token, block_table, max_pages, page_size, n, H, row, rank, scale, window, part, nslices, redo, stream)
    if (rank <= 128) { if (row <= 256) KLLM_LAT(8, 8); else KLLM_LAT(8, 0); }
    else if (rank <= 256) { if (row <= 384) KLLM_LAT(16, 12); else KLLM_LAT(16, 0); }
    else { if (row <= 576) KLLM_LAT(32, 18); else if (row <= 640) KLLM_LAT(32, 20); else KLLM_LAT(32, 0); }
#undef KLLM_LAT
    KLLM_CHECK_LAUNCH("attn_latent");
    return 0;
  }
  if (dtype == DT_F32)
    hipLaunchKernelGGL(attn_latent_kernel<float>, dim3(n, H), dim3(kLatThreads), 0, stream, (const float*)q,
                       (float*)out, (const float*)cache, positions, span_of_token, block_table, max_pages, page_size, H,
                       row, rank, scale, window);
  else
    hipLaunchKernelGGL(attn_latent_kernel<bf16_t>, dim3(n, H), dim3(kLatThreads), 0, stream, (const bf16_t*)q,
                       (bf16_t*)out, (const bf16_t*)cache, positions, span_of_token, block_table, max_pages, page_size,
                       H, row, rank, scale, window);
  KLLM_CHECK_LAUNCH("attn_latent");
  return 0;
}

extern "C" int kllm_latent_out(const void* attended, const void* w_uv, const float* gate, int nsplit, long split_stride,
                               long gate_stride, void* out, int n, int H, int dv, int rank, int dtype, int gate_by_head,
                               hipStream_t stream) {
  KLLM_REQUIRE(attended && w_uv && out, "latent_out: null pointer");
  KLLM_REQUIRE(n > 0 && H > 0 && H <= 65535 && dv > 0 && rank > 0 && rank <= 8192 && (!gate || nsplit >= 1),
               "latent_out: bad sizes n=%d H=%d dv=%d rank=%d", n, H, dv, rank);
  KLLM_REQUIRE(dtype == DT_F32 || dtype == DT_BF16, "latent_out: unknown dtype %d", dtype);
  if (dtype == DT_BF16 && n >= kLatTokens && rank % 16 == 0 && dv % 4 == 0 && ((uintptr_t)attended & 15) == 0 &&
      ((uintptr_t)w_uv & 15) == 0 && ((uintptr_t)out & 7) == 0 && (n + kLatTokens - 1) / kLatTokens <= 65535) {
    hipLaunchKernelGGL(latent_out_block_kernel, dim3(H, (n + kLatTokens - 1) / kLatTokens, (dv + 63) / 64), dim3(kLatThreads), 0,
                       stream, (const bf16_t*)attended, (const bf16_t*)w_uv, gate, nsplit, split_stride, gate_stride,
                       gate_by_head, (bf16_t*)out, n, H, dv, rank);
    KLLM_CHECK_LAUNCH("latent_out");
    return 0;
  }
  if (dtype == DT_BF16 && rank % 32 == 0 && ((uintptr_t)attended & 15) == 0 && ((uintptr_t)w_uv & 15) == 0) {
    hipLaunchKernelGGL(latent_out_mfma_kernel, dim3((n + 15) / 16, H, (dv + 63) / 64), dim3(kLatThreads), 0, stream,
                       (const bf16_t*)attended, (const bf16_t*)w_uv, gate, nsplit, split_stride, gate_stride, gate_by_head,
                       (bf16_t*)out, n, H, dv, rank);
    KLLM_CHECK_LAUNCH("latent_out");
    return 0;
  }
  const size_t lds = (size_t)rank * sizeof(float);
  if (dtype == DT_F32)
    hipLaunchKernelGGL(latent_out_kernel<float>, dim3(n, H), dim3(kLatThreads), lds, stream, (const float*)attended,
                       (const float*)w_uv, gate, nsplit, split_stride, gate_stride, gate_by_head, (float*)out, H, dv, rank);
  else
    hipLaunchKernelGGL(latent_out_kernel<bf16_t>, dim3(n, H), dim3(kLatThreads), lds, stream, (const bf16_t*)attended,
                       (const bf16_t*)w_uv, gate, nsplit, split_stride, gate_stride, gate_by_head, (bf16_t*)out, H, dv, rank);
  KLLM_CHECK_LAUNCH("latent_out");
  return 0;
}
