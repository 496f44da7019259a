// What the launches that lay out keys and values share: four numbers at a time, the bias that a product left out, and the
// write of whole runs of values by tiles.
#pragma once
#include "common.h"

typedef float f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4 load4f(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 load4f(const bf16_t* p) {
  const uint2 u = *reinterpret_cast<const uint2*>(p);
  return f32x4{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
               __uint_as_float(u.y & 0xffff0000u)};
}
__device__ __forceinline__ void store4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
__device__ __forceinline__ void store4(bf16_t* p, f32x4 v) {
  uint2 u;
  u.x = (uint32_t)f32_to_bf16(v.x).bits | ((uint32_t)f32_to_bf16(v.y).bits << 16);
  u.y = (uint32_t)f32_to_bf16(v.z).bits | ((uint32_t)f32_to_bf16(v.w).bits << 16);
  *reinterpret_cast<uint2*>(p) = u;
}

// element i of a bias that the product before did not add; BIAS: 0 none, 1 float32, 2 bfloat16 (a template
// argument, so that the loads of the bias go out beside those of the row and not behind a branch)
template <int BIAS>
__device__ __forceinline__ float bias_elem(const void* bias, size_t i) {
  if (BIAS == 0) return 0.f;
  return BIAS == 1 ? ((const float*)bias)[i] : to_f32(((const bf16_t*)bias)[i]);
}

// The values of runs of tokens, one run per sequence (tokens cu_seqlens[b] .. of sequence b lie at positions
// start[b] ..): a workgroup takes 64 positions that share a page (grid (chunks, nkv, B)), turns their rows
// [position][hd] into [hd][position] in LDS and writes every dimension's positions 16 bytes at a time, where the
// token-by-token write above would touch a cache line per dimension for two bytes.
#define VT_POS 64
template <int VEC, int BIAS>      // positions per 16-byte store; the bias as in rope_kv_write_kernel
__global__ __launch_bounds__(256) void v_write_tile_kernel(const float* __restrict__ qkv,
                                                           const void* __restrict__ bias,
                                                           const int* __restrict__ cu_seqlens,
                                                           const int* __restrict__ slots,
                                                           const int* __restrict__ start,
                                                           const int* __restrict__ block_table, int bt_stride,
                                                           act_t* __restrict__ v_pool, int page_size,
                                                           int64_t page_stride, int first, int hd, int64_t ld) {
  extern __shared__ __attribute__((aligned(16))) unsigned char vt_raw[];
  act_t* ts = (act_t*)vt_raw;                        // [hd][VT_POS + VEC]
  constexpr int TS = VT_POS + VEC;
  const int b = blockIdx.z, h = blockIdx.y;
  const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0, st = start[b];
  const int P0 = (st / VT_POS + blockIdx.x) * VT_POS;
  const int lo = max(P0, st), hi = min(P0 + VT_POS, st + n);
  if (lo >= hi) return;
  const int wave = threadIdx.x / TQ_WAVE, lane = threadIdx.x % TQ_WAVE;
  const float* src0 = qkv + (size_t)(t0 + lo - st) * ld + (size_t)(first + h) * hd;      // value row of position lo
  const size_t row_stride = (size_t)ld;
  const size_t bias0 = (size_t)(first + h) * hd;      // the bias of this value head
  if (hd % 4 == 0) {        // 16 bytes of a row per thread and turn, all of a thread's loads on their way at once
    const int q4 = hd / 4, total = (hi - lo) * q4;
#pragma unroll 8
    for (int idx = threadIdx.x; idx < total; idx += 256) {
      const int r = idx / q4, d = (idx % q4) * 4;
      const f32x4 v = load4f(src0 + r * row_stride + d);
      act_t* to = ts + d * TS + (lo + r - P0);
      to[0] = from_f32<act_t>(v.x + bias_elem<BIAS>(bias, bias0 + d));
      to[TS] = from_f32<act_t>(v.y + bias_elem<BIAS>(bias, bias0 + d + 1));
      to[2 * TS] = from_f32<act_t>(v.z + bias_elem<BIAS>(bias, bias0 + d + 2));
      to[3 * TS] = from_f32<act_t>(v.w + bias_elem<BIAS>(bias, bias0 + d + 3));
    }
  } else {
    for (int r = wave; r < hi - lo; r += 4)
      for (int d = lane; d < hd; d += TQ_WAVE)
        ts[d * TS + (lo + r - P0)] = from_f32<act_t>(src0[r * row_stride + d] + bias_elem<BIAS>(bias, bias0 + d));
  }
  __syncthreads();
  const int page = block_table[(size_t)slots[b] * bt_stride + P0 / page_size];
  act_t* base = v_pool + (size_t)page * page_stride + (size_t)h * page_size * hd + P0 % page_size;
  constexpr int GROUPS = VT_POS / VEC;
  for (int idx = threadIdx.x; idx < hd * GROUPS; idx += blockDim.x) {
    const int d = idx / GROUPS, g = idx % GROUPS;
    const int p0 = P0 + g * VEC;
    act_t* dst = base + (size_t)d * page_size + g * VEC;
    const act_t* from = ts + d * TS + g * VEC;
    if (p0 >= lo && p0 + VEC <= hi) {
      *reinterpret_cast<uint4*>(dst) = *reinterpret_cast<const uint4*>(from);
    } else {
      for (int j = max(p0, lo) - p0; j < min(p0 + VEC, hi) - p0; ++j) dst[j] = from[j];
    }
  }
}

// Whether the values of a step go by tiles: whole runs of tokens, pages of whole tiles, and a tile that fits LDS.
static inline bool value_tiles_fit(const int* cu_seqlens, const int* slots, const int* start, int B, int nkv, int hd, int max_new,
                                   int page_size) {
  constexpr int VEC = 16 / (int)sizeof(act_t);
  return cu_seqlens && slots && start && B > 0 && B <= 65535 && nkv <= 65535 && max_new > 8 && page_size % VT_POS == 0 &&
         (size_t)hd * (VT_POS + VEC) * sizeof(act_t) <= 64 * 1024;
}

// first: the head of the rows of qkv (hd numbers each) that holds the first value head.
template <int BIAS>
static void launch_value_tiles(const float* qkv, const void* bias, const int* cu_seqlens, const int* slots, const int* start,
                               const int* block_table, int bt_stride, void* v_pool, int page_size, int64_t page_stride, int first,
                               int nkv, int hd, int64_t ld, int B, int max_new, hipStream_t st) {
  constexpr int VEC = 16 / (int)sizeof(act_t);
  const size_t shmem = (size_t)hd * (VT_POS + VEC) * sizeof(act_t);
  if (shmem > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)v_write_tile_kernel<VEC, BIAS>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem);
  hipLaunchKernelGGL((v_write_tile_kernel<VEC, BIAS>), dim3((max_new + VT_POS - 1) / VT_POS + 1, nkv, B), dim3(256), shmem, st, qkv,
                     bias, cu_seqlens, slots, start, block_table, bt_stride, (act_t*)v_pool, page_size, page_stride, first, hd, ld);
}
