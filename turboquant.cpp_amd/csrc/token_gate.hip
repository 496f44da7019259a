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
