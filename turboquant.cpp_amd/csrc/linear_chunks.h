// What the chunked forms of the linear recurrences (lightning.hip, matrix_memory.hip) share: a step's runs of tokens cut
// into chunks of LC_T tokens that start at the first token the step brings for a sequence, and a chunk's rows on their way
// into LDS.
#pragma once
#include "common.h"

#define LC_T 64        // tokens of a chunk
#define LC_V 64        // value channels of a workgroup
#define LC_VLD 80      // floats between two tokens' value channels in LDS

typedef float lc_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ int lc_chunk_base(const int* __restrict__ cu_seqlens, int b) {
  int base = 0;
  for (int i = 0; i < b; ++i) base += (cu_seqlens[i + 1] - cu_seqlens[i] + LC_T - 1) / LC_T;
  return base;
}

// A chunk's rows of one projection on their way into LDS: first every load (all in flight together), then a function of
// each number and the stores.  W numbers a row (WP in LDS, a multiple of 16; zeros behind W and behind the chunk's nc tokens).  VEC: rows
// start at multiples of 16 bytes and W is a multiple of four.
template <int WP, bool VEC>
struct LcRows {
  static constexpr int N = VEC ? LC_T * WP / 4 / 256 : LC_T * WP / 256;
  float x[VEC ? 4 * N : N];
  __device__ __forceinline__ void fetch(const float* __restrict__ src, int64_t ld, int nc, int W, int tid) {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int idx = tid + 256 * i;
      if (VEC) {
        const int s = idx / (WP / 4), d = 4 * (idx % (WP / 4));
        const float4 v = s < nc && d < W ? *reinterpret_cast<const float4*>(src + (size_t)s * ld + d) : float4{0.f, 0.f, 0.f, 0.f};
        x[4 * i] = v.x, x[4 * i + 1] = v.y, x[4 * i + 2] = v.z, x[4 * i + 3] = v.w;
      } else {
        const int s = idx / WP, d = idx % WP;
        x[i] = s < nc && d < W ? src[(size_t)s * ld + d] : 0.f;
      }
    }
  }
  // dst[s * ld + d] = f(x) * (wt ? wt[s] : 1)
  template <class F>
  __device__ __forceinline__ void store(float* __restrict__ dst, int ld, const float* __restrict__ wt, int tid, F f) const {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int idx = tid + 256 * i;
      if (VEC) {
        const int s = idx / (WP / 4), d = 4 * (idx % (WP / 4));
        const float w = wt ? wt[s] : 1.f;
        *reinterpret_cast<float4*>(dst + s * ld + d) =
            float4{w * f(x[4 * i]), w * f(x[4 * i + 1]), w * f(x[4 * i + 2]), w * f(x[4 * i + 3])};
      } else {
        const int s = idx / WP, d = idx % WP;
        dst[s * ld + d] = (wt ? wt[s] : 1.f) * f(x[i]);
      }
    }
  }
  // dst[s * WP + (d ^ 16 (s % 4))] = x, WP a multiple of 64: rows without padding whose 16 columns by 4 rows lie on 64 banks
  __device__ __forceinline__ void store_turned(float* __restrict__ dst, int tid) const {
#pragma unroll
    for (int i = 0; i < N; ++i) {
      const int idx = tid + 256 * i;
      if (VEC) {
        const int s = idx / (WP / 4), d = 4 * (idx % (WP / 4));
        *reinterpret_cast<float4*>(dst + s * WP + (d ^ (16 * (s & 3)))) = float4{x[4 * i], x[4 * i + 1], x[4 * i + 2], x[4 * i + 3]};
      } else {
        const int s = idx / WP, d = idx % WP;
        dst[s * WP + (d ^ (16 * (s & 3)))] = x[i];
      }
    }
  }
};
