// A token's own vector as the other factor of an activation: out[t][j] = f(sum_s p[s][t][j]) * table[tokens[t]][j], in the
// activation type.  p: partial sums of a product, [S][T][N] float; table: rows of N numbers ld_table apart (columns of a
// wider table with a row per token of the vocabulary); f an activation of gates.def.
#include "common.h"

template <class W>
__global__ __launch_bounds__(256) void token_gate_kernel(const float* __restrict__ p, int S, size_t stride,
                                                         const int* __restrict__ tokens, const W* __restrict__ table,
                                                         int64_t ld_table, int kind, act_t* __restrict__ out, int64_t total,
                                                         int N) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int64_t t = i / N;
  const int j = (int)(i % N);
  const float e = to_f32(table[(size_t)tokens[t] * ld_table + j]);
  float v = 0.f;
  for (int s = 0; s < S; ++s) v += p[s * stride + i];
  out[i] = from_f32<act_t>(gate_fn(v, kind) * e);
}

TQ_API int tq_token_gate(const float* p, int S, const int* tokens, const void* table, int wtype, int64_t ld_table, int kind,
                         void* out, int T, int N, hipStream_t st) {
  if (T <= 0 || N <= 0) return 0;
  if (S < 1 || kind < 0 || kind >= TQ_GATE_COUNT || ld_table < N) return TQ_ERR_BAD_ARG;
  const int64_t total = (int64_t)T * N;
  if ((total + 255) / 256 > 0x7fffffff) return TQ_ERR_UNSUPPORTED;
  TQ_DISPATCH_W(wtype, {
    hipLaunchKernelGGL(token_gate_kernel<W>, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, st, p, S, (size_t)total, tokens,
                       (const W*)table, ld_table, kind, (act_t*)out, total, N);
  });
  TQ_LAUNCH_CHECK();
  return 0;
}

// The product before it in the same launch, for steps of a few tokens: out[t][j] = f(sum_k a[t][k] * w[j][k]) * table[tokens[t]][j].
// A wave (a workgroup of its own) takes a row of w for one token, grid (N, T); K in whole pieces of 16 bytes.
template <class W>
__global__ __launch_bounds__(64) void token_gate_product_kernel(const act_t* __restrict__ a, int64_t lda, const act_t* __restrict__ w,
                                                                const int* __restrict__ tokens, const W* __restrict__ table,
                                                                int64_t ld_table, int kind, act_t* __restrict__ out, int N, int K) {
  constexpr int E = 16 / (int)sizeof(act_t);
  const int j = blockIdx.x, t = blockIdx.y, lane = threadIdx.x;
  const act_t *wr = w + (size_t)j * K, *ar = a + (size_t)t * lda;
  const float e = to_f32(table[(size_t)tokens[t] * ld_table + j]);
  float acc = 0.f;
#pragma unroll 4
  for (int k = lane * E; k < K; k += 64 * E) {
    const uint4 wv = *reinterpret_cast<const uint4*>(wr + k), av = *reinterpret_cast<const uint4*>(ar + k);
    const uint32_t wu[4] = {wv.x, wv.y, wv.z, wv.w}, au[4] = {av.x, av.y, av.z, av.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if constexpr (E == 8) {
        acc = fmaf(__uint_as_float(au[i] << 16), __uint_as_float(wu[i] << 16), acc);
        acc = fmaf(__uint_as_float(au[i] & 0xffff0000u), __uint_as_float(wu[i] & 0xffff0000u), acc);
      } else {
        acc = fmaf(__uint_as_float(au[i]), __uint_as_float(wu[i]), acc);
      }
    }
  }
  acc = wave_sum(acc);
  if (lane == 0) out[(size_t)t * N + j] = from_f32<act_t>(gate_fn(acc, kind) * e);
}

TQ_API int tq_token_gate_product(const void* a, int64_t lda, const void* w, const int* tokens, const void* table, int wtype,
                                 int64_t ld_table, int kind, void* out, int T, int N, int K, hipStream_t st) {
  if (T <= 0 || N <= 0) return 0;
  constexpr int E = 16 / (int)sizeof(act_t);
  if (kind < 0 || kind >= TQ_GATE_COUNT || ld_table < N || lda < K) return TQ_ERR_BAD_ARG;
  if (T > 16 || K % E != 0 || lda % E != 0 || (uintptr_t)a % 16 != 0 || (uintptr_t)w % 16 != 0) return TQ_ERR_UNSUPPORTED;
  TQ_DISPATCH_W(wtype, {
    hipLaunchKernelGGL(token_gate_product_kernel<W>, dim3(N, T), dim3(64), 0, st, (const act_t*)a, lda, (const act_t*)w, tokens,
                       (const W*)table, ld_table, kind, (act_t*)out, N, K);
  });
  TQ_LAUNCH_CHECK();
  return 0;
}
