// What lies between the query/key/value product and attention for a mixer whose three projections
// pass a short causal convolution per channel, or have biases, or are to be padded: convolution (none
// without its weights), bias, rotation of the first `rot` elements of every query and key head,
// queries out, keys and values into pages (queries alone without a cache: KV is 0).  All in 32-bit.
//
// A wave takes a tile of tokens (16, or one in a step of single tokens) and one head of q, k or v:
// the tile's rows and the taps - 1 rows before it pass through LDS once (the sums' slices added on the
// way), the convolution runs down the columns in registers, and values are written with the tile's
// tokens as the fast index, which is how a page holds them.
//
// Pages may be wider than the heads: keys and values take `width` elements a slot, zeros beyond
// their own (so that attention's kernels, which know one width, take any pair of widths).
// Page layout: keys [KV][slot][width], then values [KV][width][slot].
#include <math.h>

#include "common.hpp"
#include "conv.hpp"
#include "kllm_kernels.h"

namespace kllm {

constexpr int kConvTile = 16;
constexpr int kConvWaves = 4;

template <typename T, int TILE>
__global__ __launch_bounds__(64 * kConvWaves) void qkv_conv_append_kernel(
    const float* __restrict__ in, int nsplit, long split_stride, long row_len, const float* __restrict__ conv_w, int taps,
    float* __restrict__ state, long slot_stride, int advance, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, int rot, int interleaved, float v_scale, T* __restrict__ q_out,
    T* __restrict__ cache, const int* __restrict__ positions, const int* __restrict__ span_of_token,
    const int* __restrict__ slots, const int* __restrict__ span_start, const int* __restrict__ span_pos,
    const int* __restrict__ block_table, int max_pages, int page_size, int n, int H, int KV, int dk, int dv, int width,
    int ld, const float* __restrict__ bias) {
  extern __shared__ float conv_lds[];                  // [waves][TILE + taps - 1][ld]
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
  const int item = blockIdx.y * kConvWaves + wave;
  const bool there = item < H + 2 * KV;
  const int K = taps - 1;
  const long first = (long)blockIdx.x * TILE;
  const int nt = (int)min((long)TILE, n - first);
  float* rows = conv_lds + (long)wave * (TILE + K) * ld;
  const bool is_v = item >= H + KV;
  const int len = is_v ? dv : dk;
  const int ch0 = !is_v ? item * dk : (H + KV) * dk + (item - H - KV) * dv;     // the head's first channel
  // lane l looks up where token l % TILE of the tile goes, before anything waits
  const long my_t = first + min(lane % TILE, nt - 1);
  const int my_pos = positions[my_t];
  const int my_page = cache ? block_table[(long)span_of_token[my_t] * max_pages + my_pos / page_size] : 0;
  const int my_slot = my_pos % page_size;
  if (there) {
    // rows before the tile may belong to other requests: then they are not looked at.  Eight rows' loads
    // go out together.
    for (int e = lane; e < len; e += kWave) {
      const float* src = in + ch0 + e;
      const float b = bias ? bias[ch0 + e] : 0.f;
      for (int r0 = 0; r0 < K + nt; r0 += 8) {
        float v[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) v[u] = b;
        for (int sl = 0; sl < nsplit; ++sl)
#pragma unroll
          for (int u = 0; u < 8; ++u) {
            const long row = min(max(first - K + r0 + u, 0L), (long)n - 1);
            v[u] += src[sl * split_stride + row * row_len];
          }
#pragma unroll
        for (int u = 0; u < 8; ++u)
          if (r0 + u < K + nt) rows[(r0 + u) * ld + e] = v[u];
      }
    }
  }
  __syncthreads();
  // Whole tiles inside one span whose earlier inputs lie in the step go down the columns; any
  // other tile asks token by token where each input is.
  const int span_first = span_of_token[first];
  const bool inside = span_of_token[first + nt - 1] == span_first && first - K >= span_start[span_first];
  if (there && conv_w) {
    for (int e = lane; e < len; e += kWave) {
      const float* w = conv_w + (long)(ch0 + e) * taps;
      float y[TILE];
#pragma unroll
      for (int tt = 0; tt < TILE; ++tt) y[tt] = 0.f;
      if (inside) {
        for (int j = 0; j < taps; ++j) {
          const float wj = w[j];
#pragma unroll
          for (int tt = 0; tt < TILE; ++tt)
            if (tt < nt) y[tt] = fmaf(wj, rows[(tt + j) * ld + e], y[tt]);
        }
      } else {
#pragma unroll
        for (int tt = 0; tt < TILE; ++tt) {
          if (tt >= nt) continue;
          const int span = span_of_token[first + tt];
          const long t0 = span_start[span];
          const bool fresh = span_pos[span] == 0;
          float* st = state + (long)slots[span] * slot_stride + (long)(ch0 + e) * K;
          float acc = 0.f;
          for (int j = 0; j < taps; ++j) {
            const long row = first + tt - K + j;
            float x;
            if (row >= t0) x = rows[(tt + j) * ld + e];
            else x = fresh ? 0.f : st[K - (int)(t0 - row)];
            acc = fmaf(w[j], x, acc);
          }
          y[tt] = acc;
          // a step of single tokens: the request's inputs move up, this lane's channel alone
          if (advance)
            for (int j = 0; j < K; ++j)
              st[j] = j + 1 < K ? (fresh ? 0.f : st[j + 1]) : rows[(tt + K) * ld + e];
        }
      }
      // (a column is this lane's own: its inputs are read, the outputs take their place)
#pragma unroll
      for (int tt = 0; tt < TILE; ++tt)
        if (tt < nt) rows[tt * ld + e] = y[tt];
    }
  }
  __syncthreads();
  if (!there) return;
  const long block = (long)page_size * width;
  if (is_v) {
    const int h = item - H - KV;
    const int tt = lane % TILE;
    if (tt >= nt) return;
    T* dst = cache + (((long)my_page * 2 + 1) * KV + h) * block + my_slot;
    for (int e = lane / TILE; e < width; e += kWave / TILE)
      dst[(long)e * page_size] = from_f32<T>(e < dv ? v_scale * rows[tt * ld + e] : 0.f);
    return;
  }
  const bool is_q = item < H;
  const int h = is_q ? item : item - H;
  const int half = rot / 2;
  for (int e = lane; e < width; e += kWave) {
    // which element turns with this one, and which way: the same for every token of the tile
    const bool turns = cos_t && e < rot;
    int j = 0, partner = 0;
    bool lead = true;
    if (turns) {
      if (interleaved) {
        j = e / 2;
        lead = (e & 1) == 0;
        partner = lead ? e + 1 : e - 1;
      } else {
        lead = e < half;
        j = lead ? e : e - half;
        partner = lead ? e + half : e - half;
      }
    }
    float cs[TILE], sn[TILE];
#pragma unroll
    for (int tt = 0; tt < TILE; ++tt) {
      const long at = (first + min(tt, nt - 1)) * half + j;
      cs[tt] = turns ? cos_t[at] : 1.f;
      sn[tt] = turns ? sin_t[at] : 0.f;
    }
#pragma unroll
    for (int tt = 0; tt < TILE; ++tt) {
      if (tt >= nt) continue;
      const float v = e < dk ? rows[tt * ld + e] : 0.f;
      const float o = turns ? rows[tt * ld + partner] : 0.f;
      const float r = lead ? v * cs[tt] - o * sn[tt] : v * cs[tt] + o * sn[tt];
      T* dst = is_q ? q_out + ((first + tt) * H + h) * width
                    : cache + ((long)__builtin_amdgcn_readlane(my_page, tt) * 2 * KV + h) * block +
                          (long)__builtin_amdgcn_readlane(my_slot, tt) * width;
      dst[e] = from_f32<T>(r);
    }
  }
}

}  // namespace kllm

using namespace kllm;

extern "C" int kllm_qkv_conv_append(const float* sums, int nsplit, long split_stride, int row_len, int col0,
                                    const float* conv_w, int taps, float* state, long slot_stride, int single,
                                    const float* cos_t, const float* sin_t, int rot, int interleaved, float v_scale,
                                    void* q_out, void* cache, const int* positions, const int* span_of_token,
                                    const int* slots, const int* span_start, const int* span_pos,
                                    const int* block_table, int max_pages, int page_size, int n, int H, int KV, int dk,
                                    int dv, int width, int dtype, const float* bias, hipStream_t stream) {
  KLLM_REQUIRE(sums && q_out && positions && span_of_token && slots && span_start && span_pos && block_table,
               "qkv_conv_append: null pointer");
  KLLM_REQUIRE((conv_w || taps == 1) && (!conv_w || !bias), "qkv_conv_append: a convolution has weights and no bias in front of it");
  KLLM_REQUIRE(n > 0 && H > 0 && (cache ? KV > 0 : KV == 0) && dk > 0 && dv > 0 && dk <= width && dv <= width && nsplit >= 1 && col0 >= 0 &&
                   col0 + (H + KV) * dk + KV * dv <= row_len,
               "qkv_conv_append: bad sizes n=%d H=%d KV=%d dk=%d dv=%d width=%d row=%d", n, H, KV, dk, dv, width, row_len);
  KLLM_REQUIRE(taps >= 1 && taps <= kMaxTaps && (taps == 1 || state), "qkv_conv_append: %d taps (1 to %d), with their state",
               taps, kMaxTaps);
  KLLM_REQUIRE((cos_t == nullptr) == (sin_t == nullptr) && (!cos_t || (rot > 0 && rot % 2 == 0 && rot <= dk)),
               "qkv_conv_append: rotary dimension %d of a head of %d", rot, dk);
  KLLM_REQUIRE(max_pages > 0 && page_size > 0 && (dtype == DT_F32 || dtype == DT_BF16), "qkv_conv_append: bad cache or dtype");
  const int tile = single ? 1 : kConvTile;
  const int ld = (dk > dv ? dk : dv) + 1;
  const size_t lds = (size_t)kConvWaves * (tile + taps - 1) * ld * sizeof(float);
  KLLM_REQUIRE(lds <= 160 * 1024, "qkv_conv_append: heads of %d and %d do not fit into LDS", dk, dv);
  const dim3 grid(ceil_div(n, tile), ceil_div(H + 2 * KV, kConvWaves));
  KLLM_REQUIRE(grid.y <= 65535, "qkv_conv_append: too many heads for the grid");
#define KLLM_QC(T, TILE)                                                                                               \
  do {                                                                                                                 \
    if (lds > 64 * 1024)                                                                                               \
      (void)hipFuncSetAttribute((const void*)qkv_conv_append_kernel<T, TILE>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
    hipLaunchKernelGGL((qkv_conv_append_kernel<T, TILE>), grid, dim3(64 * kConvWaves), lds, stream, sums + col0, nsplit, \
                       split_stride, (long)row_len, conv_w, taps, state, slot_stride, single && taps > 1 ? 1 : 0, cos_t, sin_t, \
                       rot, interleaved, v_scale, (T*)q_out, (T*)cache, positions, span_of_token, slots, span_start,   \
                       span_pos, block_table, max_pages, page_size, n, H, KV, dk, dv, width, ld, bias);                \
  } while (0)
  if (dtype == DT_F32) {
    if (single) KLLM_QC(float, 1); else KLLM_QC(float, kConvTile);
  } else {
    if (single) KLLM_QC(bf16_t, 1); else KLLM_QC(bf16_t, kConvTile);
  }
#undef KLLM_QC
  KLLM_CHECK_LAUNCH("qkv_conv_append");
  return 0;
}
