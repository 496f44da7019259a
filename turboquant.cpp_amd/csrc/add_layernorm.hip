// The residual sum with norms that take the mean off (layer norms), for what is added and for the stream, in one pass.
//
// For row r (token rows[r], or r itself when rows is null):
//   d = what a part left: partial sums delta[s][row] added up in order, or, with y set, the experts' unsummed rows
//       sum_j weights[row][j] * y[pair_slot[row][j]] (j ascending; a slot of -1: no row) + gate[row] * sum_s delta[s][row];
//       neither: nothing is added
//   d <- norm_d(d)            kind 0: as it is; 1: d / sqrt(mean(d^2) + eps) * wd;
//                             2: with c = d - mean(d), c / sqrt(mean(c^2) + eps) * wd + bd
//   v = x[row] + d            written back to x when rows is null
//   out = norm(v)             kind 0: the summed stream itself; 1 and 2 as above, with w and b
// A row waits in registers between the sums (a thread has NV runs of N neighbouring numbers), so it is read once and written
// once.  The order of every sum depends on H alone.
#include "value_tiles.h"

struct AddNormArgs {
  float* x;
  const float* delta;
  int S;
  size_t delta_stride;
  const float* y;
  const int* pair_slot;
  const float* weights;
  int topk;
  const float* gate;
  int kind_d, kind;
  const void *wd, *bd, *w, *b;
  float eps_d, eps;
  const int* rows;
  act_t* out;
  float* out32;
  int H;
};

template <int N>
struct Run {
  float v[N];
};
template <int N, class T>
__device__ __forceinline__ Run<N> load_run(const T* p) {
  Run<N> r;
  if constexpr (N == 4) {
    const f32x4 t = load4f(p);
    r.v[0] = t.x, r.v[1] = t.y, r.v[2] = t.z, r.v[3] = t.w;
  } else {
    r.v[0] = to_f32(*p);
  }
  return r;
}
template <int N, class T>
__device__ __forceinline__ void store_run(T* p, const Run<N>& r) {
  if constexpr (N == 4) store4(p, f32x4{r.v[0], r.v[1], r.v[2], r.v[3]});
  else *p = from_f32<T>(r.v[0]);
}

// v <- norm of the row that the workgroup's threads hold in v
template <class W, int N, int NV>
__device__ __forceinline__ void norm_row(Run<N> (&v)[NV], int kind, const W* w, const W* b, float eps, int H, float* red) {
  const int step = blockDim.x * N, i0 = threadIdx.x * N;
  if (kind == 2) {
    float s = 0.f;
#pragma unroll
    for (int u = 0; u < NV; ++u)
#pragma unroll
      for (int e = 0; e < N; ++e) s += v[u].v[e];      // (numbers beyond the row are zeros)
    const float mean = block_sum(s, red) / (float)H;
#pragma unroll
    for (int u = 0; u < NV; ++u)
#pragma unroll
      for (int e = 0; e < N; ++e) v[u].v[e] = i0 + u * step < H ? v[u].v[e] - mean : 0.f;
  }
  float ss = 0.f;
#pragma unroll
  for (int u = 0; u < NV; ++u)
#pragma unroll
    for (int e = 0; e < N; ++e) ss = fmaf(v[u].v[e], v[u].v[e], ss);
  const float rs = 1.0f / sqrtf(block_sum(ss, red) / (float)H + eps);
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int i = i0 + u * step;
    if (i < H) {
      const Run<N> wt = load_run<N>(w + i);
#pragma unroll
      for (int e = 0; e < N; ++e) v[u].v[e] = v[u].v[e] * rs * wt.v[e];
      if (kind == 2) {
        const Run<N> bt = load_run<N>(b + i);
#pragma unroll
        for (int e = 0; e < N; ++e) v[u].v[e] += bt.v[e];
      }
    }
  }
}

template <class W, int N, int NV>
__global__ void add_norm_kernel(AddNormArgs a) {
  __shared__ float red[1024 / TQ_WAVE];
  __shared__ int slot[64];
  __shared__ float wgt[64];
  const int r = blockIdx.x, H = a.H;
  const int row = a.rows ? a.rows[r] : r;
  const int step = blockDim.x * N, i0 = threadIdx.x * N;
  float* xr = a.x + (size_t)row * H;
  const float* dr = a.delta + (size_t)row * H;
  Run<N> x[NV], d[NV];
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int i = i0 + u * step;
#pragma unroll
    for (int e = 0; e < N; ++e) x[u].v[e] = d[u].v[e] = 0.f;
    if (i < H) x[u] = load_run<N>(xr + i);
  }
  float g = 1.0f;
  if (a.y) {
    if ((int)threadIdx.x < a.topk) {
      slot[threadIdx.x] = a.pair_slot[(size_t)row * a.topk + threadIdx.x];
      wgt[threadIdx.x] = a.weights[(size_t)row * a.topk + threadIdx.x];
    }
    if (a.gate) g = a.gate[row];
    __syncthreads();
  }
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int i = i0 + u * step;
    if (i >= H) continue;
    // the terms are fetched four at a time and added in their order
    for (int s = 0; s < a.S; s += 4) {
      Run<N> t[4];
#pragma unroll
      for (int k = 0; k < 4; ++k)
        if (s + k < a.S) t[k] = load_run<N>(dr + (s + k) * a.delta_stride + i);
#pragma unroll
      for (int k = 0; k < 4; ++k)
        if (s + k < a.S)
#pragma unroll
          for (int e = 0; e < N; ++e) d[u].v[e] += t[k].v[e];
    }
    if (a.y) {
      Run<N> acc;
#pragma unroll
      for (int e = 0; e < N; ++e) acc.v[e] = 0.f;
      for (int j = 0; j < a.topk; j += 4) {
        Run<N> t[4];
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (j + k < a.topk && slot[j + k] >= 0) t[k] = load_run<N>(a.y + (size_t)slot[j + k] * H + i);
#pragma unroll
        for (int k = 0; k < 4; ++k)
          if (j + k < a.topk && slot[j + k] >= 0)
#pragma unroll
            for (int e = 0; e < N; ++e) acc.v[e] = fmaf(wgt[j + k], t[k].v[e], acc.v[e]);
      }
#pragma unroll
      for (int e = 0; e < N; ++e) d[u].v[e] = fmaf(g, d[u].v[e], acc.v[e]);
    }
  }
  if (a.kind_d) norm_row<W, N, NV>(d, a.kind_d, (const W*)a.wd, (const W*)a.bd, a.eps_d, H, red);
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int i = i0 + u * step;
#pragma unroll
    for (int e = 0; e < N; ++e) x[u].v[e] += d[u].v[e];
    if (i < H && !a.rows) store_run<N>(xr + i, x[u]);
  }
  if (a.kind) norm_row<W, N, NV>(x, a.kind, (const W*)a.w, (const W*)a.b, a.eps, H, red);
#pragma unroll
  for (int u = 0; u < NV; ++u) {
    const int i = i0 + u * step;
    if (i < H && a.out) store_run<N>(a.out + (size_t)r * H + i, x[u]);
    if (i < H && a.out32) store_run<N>(a.out32 + (size_t)r * H + i, x[u]);
  }
}

// kind_d, kind: 0 none, 1 root mean square (wd / w), 2 layer norm (wd, bd / w, b).  delta null and y null: nothing is added
// (kind_d 0).  out, out32 (either may be null): the normed rows, or with kind 0 the summed stream.  Rows of up to 32,768
// numbers.
TQ_API int tq_add_norm(float* x, const float* delta, int S, int64_t delta_stride, const float* y, const int* pair_slot,
                       const float* weights, int topk, const float* gate, int kind_d, const void* wd, const void* bd, float eps_d,
                       int kind, const void* w, const void* b, float eps, int wtype, const int* rows, int R, void* out,
                       float* out32, int H, hipStream_t st) {
  if (R <= 0) return 0;
  if (kind_d < 0 || kind_d > 2 || kind < 0 || kind > 2 || (kind_d && !wd) || (kind_d == 2 && !bd) || (kind && !w) ||
      (kind == 2 && !b))
    return TQ_ERR_BAD_ARG;
  if (y && (topk < 1 || topk > 64 || !pair_slot || !weights)) return TQ_ERR_BAD_ARG;
  if (S < 0 || (S > 0 && !delta) || (kind_d && !y && S < 1)) return TQ_ERR_BAD_ARG;
  if (H < 1 || H > 32768) return TQ_ERR_UNSUPPORTED;
  const AddNormArgs a{x, delta, S, (size_t)delta_stride, y, pair_slot, weights, topk, gate, kind_d, kind, wd, bd, w, b, eps_d, eps,
                      rows, (act_t*)out, out32, H};
  const bool vec = H % 4 == 0;
  const int runs = vec ? H / 4 : H;
  // a function of H alone: a row's sums do not depend on what else the step holds
  const int threads = runs >= 4096 ? 1024 : runs >= 512 ? 512 : 256;
  const int nv = (runs + threads - 1) / threads;
#define TQ_AN(NN, NVV) hipLaunchKernelGGL((add_norm_kernel<W, NN, NVV>), dim3(R), dim3(threads), 0, st, a)
  TQ_DISPATCH_W(wtype, {
    if (vec) {
      if (nv <= 1) TQ_AN(4, 1);
      else if (nv <= 2) TQ_AN(4, 2);
      else if (nv <= 4) TQ_AN(4, 4);
      else TQ_AN(4, 8);
    } else {
      if (nv <= 4) TQ_AN(1, 4);
      else TQ_AN(1, 32);
    }
  });
#undef TQ_AN
  TQ_LAUNCH_CHECK();
  return 0;
}
