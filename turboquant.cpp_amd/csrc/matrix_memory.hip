// A matrix memory with exponential gates (the mLSTM cell), over per-sequence state of fixed size.
//
// Per head, with a state S [D][V] (key channels by value channels), a normaliser n [D] and a running maximum m that all
// start at zero, token by token:
//   i = cap tanh((raw_i + b_i) / cap),  f = logsigmoid(cap tanh((raw_f + b_f) / cap))         (logarithms of the gates)
//   m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n <- the same with k alone
//   o = S^T (q D^-1/2) / (max(|n . q D^-1/2|, e^(-m')) + 1e-6)
// with q, k (D per head), v (V per head) and the raw gates (one number per head each) projections.  Every head's read-out is
// then divided by its root mean square over V, multiplied by a weight per channel and by sigmoid(g), g a projection of its
// own.  Everything here is float arithmetic on both libraries (sums of gate logarithms over a chunk in double); the products
// around it are the library's.
//
// Projections P [T][ldp] (float): q (H D) | k (H D) | v (H V) | g (H V) | raw_i (H) | raw_f (H).
// bias (float): b_i (H) | b_f (H).   A sequence's row of state (float): S as [H][D][V], n as [H][D], m as [H].
//
// Three ways through a step, with the same formulas:
//   mm_decode    one token per sequence: a workgroup a (sequence, head), everything up to the gated output in one launch.
//   mm_scan      short runs: the recurrence over a run's tokens in order, the state in registers (MM_ROWS key channels of a
//                value channel per lane; n rides as one more value channel whose value is always 1), then mm_out.
//   mm_chunked   long runs in chunks of LC_T tokens on the matrix cores in float: see below; then mm_out.
#include "linear_chunks.h"

#define MM_ROWS 16        // key channels of a value channel that one lane keeps
#define MM_CHUNK(L) ((L) > 16 ? 4 : 16)       // tokens staged at a time
#define MM_SEG 20         // floats between the rows of two lanes in LDS
#define MM_EPS 1e-6f      // added to the read-out's denominator

// The logarithms of both gates from their projections.
__device__ __forceinline__ void mm_gates(float raw_i, float raw_f, float bi, float bf, float cap, float& i, float& f) {
  i = cap * tanhf((raw_i + bi) / cap);
  const float z = cap * tanhf((raw_f + bf) / cap);
  f = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

// Inclusive sum and running maximum over a wave's lanes.
__device__ __forceinline__ double mm_scan_sum(double x, int lane) {
#pragma unroll
  for (int o = 1; o < TQ_WAVE; o <<= 1) {
    const double up = __shfl_up(x, o, TQ_WAVE);
    if (lane >= o) x += up;
  }
  return x;
}
__device__ __forceinline__ double mm_scan_max(double x, int lane) {
#pragma unroll
  for (int o = 1; o < TQ_WAVE; o <<= 1) {
    const double up = __shfl_up(x, o, TQ_WAVE);
    if (lane >= o) x = fmax(x, up);
  }
  return x;
}

struct MmScaled {
  float s;
  __device__ __forceinline__ float operator()(float x) const { return x * s; }
};

// ------------------------------------------------------------------------------------------ short runs
// grid (ceil((V + 1) / VB), H, B), block 256; L = lanes per value channel (a power of two, L * MM_ROWS >= D), VB = 256 / L.
// Channel V is the normaliser.  num [T][H V] gets the numerators, den and mrow [T][H] the denominators and running maxima.
// (m is read by every workgroup of a head and written by none: mm_out stores it.)
template <int L>
__global__ __launch_bounds__(256) void mm_scan_kernel(const float* __restrict__ P, int64_t ldp, const float* __restrict__ bias,
                                                      float cap, const int* __restrict__ cu_seqlens,
                                                      const int* __restrict__ slots, float* __restrict__ state,
                                                      int64_t state_stride, int H, int D, int V, float* __restrict__ num,
                                                      float* __restrict__ den, float* __restrict__ mrow) {
  constexpr int VB = 256 / L, CH = MM_CHUNK(L);
  __shared__ float qs[CH][L * MM_SEG], ks[CH][L * MM_SEG], vs[CH][VB];
  __shared__ float keep_s[CH], add_s[CH], m_s[CH];
  const int b = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * VB;
  const int tid = threadIdx.x, vc = tid / L, j = tid % L;
  const int v = v0 + vc;
  const bool live = v <= V, norm = v == V;
  const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
  if (n <= 0) return;
  float* srow = state + (size_t)slots[b] * state_stride;
  float* at = norm ? srow + (size_t)H * D * V + (size_t)h * D : srow + (size_t)h * D * V + v;      // key channel d at at[d * step]
  const size_t step = norm ? 1 : V;
  float m = srow[(size_t)H * D * V + (size_t)H * D + h];
  float S[MM_ROWS];
#pragma unroll
  for (int r = 0; r < MM_ROWS; ++r) {
    const int d = j * MM_ROWS + r;
    S[r] = live && d < D ? at[(size_t)d * step] : 0.f;
  }
  const float scale = 1.0f / sqrtf((float)D), bi = bias[h], bf = bias[H + h];
  const float* q0 = P + (size_t)h * D;
  const float* k0 = P + (size_t)H * D + (size_t)h * D;
  const float* vv0 = P + (size_t)2 * H * D + (size_t)h * V + v0;
  const float* g0 = P + (size_t)2 * H * D + (size_t)2 * H * V + h;
  for (int c0 = 0; c0 < n; c0 += CH) {
    const int nc = min(CH, n - c0);
    __syncthreads();
    for (int idx = tid; idx < nc * L * MM_ROWS; idx += 256) {
      const int c = idx / (L * MM_ROWS), d = idx % (L * MM_ROWS);
      const size_t row = (size_t)(t0 + c0 + c) * ldp;
      const int to = (d / MM_ROWS) * MM_SEG + d % MM_ROWS;
      qs[c][to] = d < D ? scale * q0[row + d] : 0.f;
      ks[c][to] = d < D ? k0[row + d] : 0.f;
    }
    for (int idx = tid; idx < nc * VB; idx += 256) {
      const int c = idx / VB, i = idx % VB;
      vs[c][i] = v0 + i < V ? vv0[(size_t)(t0 + c0 + c) * ldp + i] : v0 + i == V ? 1.f : 0.f;
    }
    if (tid < TQ_WAVE) {      // every wave would find the same: one does it
      float gi = 0.f, gf = 0.f;
      if (tid < nc) mm_gates(g0[(size_t)(t0 + c0 + tid) * ldp], g0[(size_t)(t0 + c0 + tid) * ldp + H], bi, bf, cap, gi, gf);
      // m_t = F_t + max(m, max_{s <= t} (i_s - F_s)), F the running sum of f
      const double F = mm_scan_sum(tid < nc ? (double)gf : 0.0, tid);
      const double M = fmax((double)m, mm_scan_max(tid < nc ? (double)gi - F : -1e300, tid));
      const double before = __shfl_up(M, 1, TQ_WAVE);
      if (tid < nc) {
        keep_s[tid] = expf((float)((tid ? before : (double)m) - M));
        add_s[tid] = expf((float)((double)gi - F - M));
        m_s[tid] = (float)(F + M);
      }
    }
    __syncthreads();
    m = m_s[nc - 1];
    for (int c = 0; c < nc; ++c) {
      const float keep = keep_s[c], val = add_s[c] * vs[c][vc];
      const float* kr = &ks[c][j * MM_SEG];
      const float* qr = &qs[c][j * MM_SEG];
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < MM_ROWS; ++r) {
        S[r] = fmaf(keep, S[r], kr[r] * val);
        acc = fmaf(S[r], qr[r], acc);
      }
#pragma unroll
      for (int off = L / 2; off > 0; off >>= 1) acc += __shfl_xor(acc, off, TQ_WAVE);
      if (j == 0 && live) {
        const size_t th = (size_t)(t0 + c0 + c) * H + h;
        if (norm) {
          den[th] = fmaxf(fabsf(acc), expf(-m_s[c])) + MM_EPS;
          mrow[th] = m_s[c];
        } else {
          num[th * V + v] = acc;
        }
      }
    }
  }
  if (live) {
#pragma unroll
    for (int r = 0; r < MM_ROWS; ++r) {
      const int d = j * MM_ROWS + r;
      if (d < D) at[(size_t)d * step] = S[r];
    }
  }
}

// P: the step's projections [T][ldp]; cu_seqlens [B + 1], slots [B]: the tokens as one run per sequence; state: the rows of
// all slots, state_stride floats apart; num [T][H V], den, mrow [T][H] float.  The rows' m stays as it was: tq_mm_out
// writes it.
TQ_API int tq_mm_scan(const float* P, int64_t ldp, const float* bias, float cap, const int* cu_seqlens, const int* slots,
                      float* state, int64_t state_stride, int B, int H, int D, int V, float* num, float* den, float* mrow,
                      hipStream_t st) {
  if (B <= 0) return 0;
  if (H < 1 || D < 1 || V < 1 || ldp < (int64_t)2 * H * (D + V + 1) || state_stride < (int64_t)H * ((int64_t)D * V + D + 1) ||
      !(cap > 0.f) || !bias || !num || !den || !mrow)
    return TQ_ERR_BAD_ARG;
  if (D > 64 * MM_ROWS || H > 65535 || B > 65535) return TQ_ERR_UNSUPPORTED;
  int L = 1;
  while (L * MM_ROWS < D) L *= 2;
#define TQ_MM_LAUNCH(LV)                                                                                                   \
  hipLaunchKernelGGL(mm_scan_kernel<LV>, dim3((V + 1 + 256 / LV - 1) / (256 / LV), H, B), dim3(256), 0, st, P, ldp, bias,  \
                     cap, cu_seqlens, slots, state, state_stride, H, D, V, num, den, mrow)
  switch (L) {
    case 1: TQ_MM_LAUNCH(1); break;
    case 2: TQ_MM_LAUNCH(2); break;
    case 4: TQ_MM_LAUNCH(4); break;
    case 8: TQ_MM_LAUNCH(8); break;
    case 16: TQ_MM_LAUNCH(16); break;
    case 32: TQ_MM_LAUNCH(32); break;
    default: TQ_MM_LAUNCH(64); break;
  }
#undef TQ_MM_LAUNCH
  TQ_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------------------------------ long runs, in chunks
// With F_t the sum of f over a chunk's tokens up to t, a_s = i_s - F_s, m the running maximum before the chunk, S and n the
// state before it, and M_t = max(m, max_{s <= t} a_s) (so that the running maximum at t is F_t + M_t):
//   numerator_t = sum_{s <= t} e^(a_s - M_t) (q_t . k_s) v_s + e^(m - M_t) S^T q_t,       n . q likewise without the values
// and at the chunk's end, with A = max_s a_s over its tokens:
//   state' = e^(m - M) state + e^(A - M) sum_s e^(a_s - A) k_s v_s^T,   m' = F + M,  M = max(m, A)
// No exponent is positive.  Three launches: every chunk's own sum (chunks side by side) with its F and A; the states before
// the chunks, per element over a sequence's chunks in order (the sequence's row of state is read first and written last);
// every chunk's numerators and denominators, the last chunk's also the new m.  F, a and M are kept in double: a chunk's F may
// reach some hundreds, of which differences are taken.
//
// scratch (float): per chunk H (D V + D) floats, [H][D V] then [H][D]; scal (double): per chunk and head F, A and, from the second
// launch on, the m before the chunk.

// grid (ceil(V / LC_V), H, B * NC), block 256: a wave to 16 value channels.
template <int ND, bool VEC>
__global__ __launch_bounds__(256) void mm_chunk_state_kernel(const float* __restrict__ P, int64_t ldp,
                                                             const float* __restrict__ bias, float cap,
                                                             const int* __restrict__ cu_seqlens, int NC, int max_chunks, int H,
                                                             int D, int V, float* __restrict__ scratch,
                                                             double* __restrict__ scal) {
  extern __shared__ __align__(16) float mm_lds[];
  constexpr int DP = 16 * ND, KLD = DP + (80 - DP % 64) % 64;
  float* ks = mm_lds;                    // [LC_T][KLD]
  float* vs = ks + LC_T * KLD;           // [LC_T][LC_VLD], each token's values times its weight
  float* wt = vs + LC_T * LC_VLD;        // [LC_T]
  const int b = blockIdx.z / NC, c = blockIdx.z % NC, h = blockIdx.y, v0 = blockIdx.x * LC_V;
  const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
  if (c * LC_T >= n) return;
  const int gi = lc_chunk_base(cu_seqlens, b) + c;
  if (gi >= max_chunks) return;
  const int nc = min(LC_T, n - c * LC_T), tid = threadIdx.x;
  const float* row0 = P + (size_t)(t0 + c * LC_T) * ldp;
  LcRows<DP, VEC> kr_;
  LcRows<LC_V, VEC> vr_;
  kr_.fetch(row0 + (size_t)H * D + (size_t)h * D, ldp, nc, D, tid);
  vr_.fetch(row0 + (size_t)2 * H * D + (size_t)h * V + v0, ldp, nc, V - v0, tid);
  if (tid < TQ_WAVE) {
    const float* g0 = row0 + (size_t)2 * H * (D + V) + h;
    float i = 0.f, f = 0.f;
    if (tid < nc) mm_gates(g0[(size_t)tid * ldp], g0[(size_t)tid * ldp + H], bias[h], bias[H + h], cap, i, f);
    const double F = mm_scan_sum(tid < nc ? (double)f : 0.0, tid);
    const double a = tid < nc ? (double)i - F : -1e300;
    const double A = __shfl(mm_scan_max(a, tid), TQ_WAVE - 1, TQ_WAVE);
    wt[tid] = tid < nc ? expf((float)(a - A)) : 0.f;
    if (blockIdx.x == 0 && tid == TQ_WAVE - 1) {
      double* sc = scal + ((size_t)gi * H + h) * 3;
      sc[0] = F;
      sc[1] = A;
    }
  }
  kr_.store(ks, KLD, nullptr, tid, MmScaled{1.f});
  __syncthreads();
  vr_.store(vs, LC_VLD, wt, tid, MmScaled{1.f});
  __syncthreads();
  const int wave = tid / 64, lane = tid % 64, g = lane / 16, r = lane % 16;
  lc_f32x4 acc[ND];
#pragma unroll
  for (int i = 0; i < ND; ++i) acc[i] = lc_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k4 = 0; k4 < LC_T / 4; ++k4) {
    const float bv = vs[(4 * k4 + g) * LC_VLD + 16 * wave + r];
    const float* kr = ks + (4 * k4 + g) * KLD + r;
#pragma unroll
    for (int rt = 0; rt < ND; ++rt) acc[rt] = __builtin_amdgcn_mfma_f32_16x16x4f32(kr[16 * rt], bv, acc[rt], 0, 0, 0);
  }
  float* chunk = scratch + (size_t)gi * H * (D * V + D);
  const int v = v0 + 16 * wave + r;
  if (v < V) {
    float* out = chunk + (size_t)h * D * V + v;
#pragma unroll
    for (int rt = 0; rt < ND; ++rt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * rt + 4 * g + i;
        if (d < D) out[(size_t)d * V] = acc[rt][i];
      }
  }
  if (blockIdx.x == 0 && tid < D) {      // (D <= 256)
    float s = 0.f;
#pragma unroll 8
    for (int t = 0; t < LC_T; ++t) s = fmaf(wt[t], ks[t * KLD + tid], s);
    chunk[(size_t)H * D * V + (size_t)h * D + tid] = s;
  }
}

// grid (ceil((D V + D) / 256), H, B), block 256: every chunk's own sums become the state before it, in place; the row of
// state (S and n) is advanced, its m is only read.
#define MM_AHEAD 16       // chunks whose sums are asked for before the first of them is replaced
__global__ __launch_bounds__(256) void mm_chunk_prefix_kernel(const int* __restrict__ cu_seqlens, const int* __restrict__ slots,
                                                              float* __restrict__ state, int64_t state_stride, int max_chunks,
                                                              int H, int D, int V, float* __restrict__ scratch,
                                                              double* __restrict__ scal) {
  const int b = blockIdx.z, h = blockIdx.y;
  const int e = blockIdx.x * 256 + threadIdx.x;
  const int n = cu_seqlens[b + 1] - cu_seqlens[b];
  if (n <= 0 || e >= D * V + D) return;
  const int base = lc_chunk_base(cu_seqlens, b), chunks = (n + LC_T - 1) / LC_T;
  if (base + chunks > max_chunks) return;
  const size_t chunk_floats = (size_t)H * (D * V + D);
  const size_t off = e < D * V ? (size_t)h * D * V + e : (size_t)H * D * V + (size_t)h * D + (e - D * V);
  float* srow = state + (size_t)slots[b] * state_stride;
  double m = srow[(size_t)H * D * V + (size_t)H * D + h];
  float carry = srow[off];
  float* at = scratch + (size_t)base * chunk_floats + off;
  double* sc = scal + ((size_t)base * H + h) * 3;
  for (int c0 = 0; c0 < chunks; c0 += MM_AHEAD) {
    float own[MM_AHEAD];
    double F[MM_AHEAD], A[MM_AHEAD];
#pragma unroll
    for (int u = 0; u < MM_AHEAD; ++u) {
      const int c = min(c0 + u, chunks - 1);
      own[u] = at[(size_t)c * chunk_floats];
      F[u] = sc[(size_t)c * H * 3];
      A[u] = sc[(size_t)c * H * 3 + 1];
    }
#pragma unroll
    for (int u = 0; u < MM_AHEAD; ++u) {
      const int c = c0 + u;
      if (c < chunks) {
        at[(size_t)c * chunk_floats] = carry;
        if (e == 0) sc[(size_t)c * H * 3 + 2] = m;
        const double M = fmax(m, A[u]);
        carry = fmaf(expf((float)(m - M)), carry, expf((float)(A[u] - M)) * own[u]);
        m = F[u] + M;
      }
    }
  }
  srow[off] = carry;
}

// grid (ceil(V / LC_V), H, B * NC), block 256: a chunk's numerators for LC_V value channels, a wave to 16 tokens; the first
// block of value channels also the denominators, and in a run's last chunk the sequence's new m.
// (the values wait in registers until the keys have been read and take their place in LDS: with key widths of up to 128 two
// workgroups fit a compute unit)
template <int ND, bool VEC>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(ND > 8 ? 1 : 2))) void mm_chunk_out_kernel(const float* __restrict__ P, int64_t ldp,
                                                           const float* __restrict__ bias, float cap,
                                                           const int* __restrict__ cu_seqlens, const int* __restrict__ slots,
                                                           float* __restrict__ state, int64_t state_stride, int NC,
                                                           int max_chunks, int H, int D, int V,
                                                           const float* __restrict__ scratch, const double* __restrict__ scal,
                                                           float* __restrict__ num, float* __restrict__ den) {
  extern __shared__ __align__(16) float mm_lds[];
  constexpr int DP = 16 * ND, QLD = DP + 4, PLD = LC_T + 4;
  double* as = reinterpret_cast<double*>(mm_lds);      // [LC_T] a_s
  double* Ms = as + LC_T;                // [LC_T] M_t
  float* coef = reinterpret_cast<float*>(Ms + LC_T);   // [LC_T] e^(m - M_t)
  float* mt = coef + LC_T;               // [LC_T] the running maximum at t
  float* qs = mt + LC_T;                 // [LC_T][QLD]
  float* ks = qs + LC_T * QLD;           // [LC_T][QLD]; later the weighted scores [LC_T][PLD]
  float* vs = ks + LC_T * PLD;           // and the values [LC_T][LC_V] behind them
  const int b = blockIdx.z / NC, c = blockIdx.z % NC, h = blockIdx.y, v0 = blockIdx.x * LC_V;
  const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
  if (c * LC_T >= n) return;
  const int gi = lc_chunk_base(cu_seqlens, b) + c;
  if (gi >= max_chunks) return;
  const int nc = min(LC_T, n - c * LC_T), tid = threadIdx.x;
  const int wave = tid / 64, lane = tid % 64, g = lane / 16, r = lane % 16;
  const float* chunk = scratch + (size_t)gi * H * (D * V + D);
  // the state before the chunk, as the last product's operand: asked for first, so that it arrives while the rest is staged
  constexpr int AHEAD = DP / 4 > 16 ? 16 : DP / 4;
  const float* sb = chunk + (size_t)h * D * V + v0 + r;
  float sv[AHEAD][4];
#pragma unroll
  for (int k4 = 0; k4 < AHEAD; ++k4)
#pragma unroll
    for (int cv = 0; cv < 4; ++cv)
      sv[k4][cv] = 4 * k4 + g < D && v0 + 16 * cv + r < V ? sb[(size_t)(4 * k4 + g) * V + 16 * cv] : 0.f;
  const float* row0 = P + (size_t)(t0 + c * LC_T) * ldp;
  LcRows<LC_V, VEC> vr_;
  {
    LcRows<DP, VEC> qr_, kr_;
    qr_.fetch(row0 + (size_t)h * D, ldp, nc, D, tid);
    kr_.fetch(row0 + (size_t)H * D + (size_t)h * D, ldp, nc, D, tid);
    vr_.fetch(row0 + (size_t)2 * H * D + (size_t)h * V + v0, ldp, nc, V - v0, tid);
    if (tid < TQ_WAVE) {
      const float* g0 = row0 + (size_t)2 * H * (D + V) + h;
      const double m = scal[((size_t)gi * H + h) * 3 + 2];
      float i = 0.f, f = 0.f;
      if (tid < nc) mm_gates(g0[(size_t)tid * ldp], g0[(size_t)tid * ldp + H], bias[h], bias[H + h], cap, i, f);
      const double F = mm_scan_sum(tid < nc ? (double)f : 0.0, tid);
      const double a = tid < nc ? (double)i - F : -1e300;
      const double M = fmax(m, mm_scan_max(a, tid));
      as[tid] = a;
      Ms[tid] = M;
      coef[tid] = expf((float)(m - M));
      mt[tid] = (float)(F + M);
    }
    qr_.store(qs, QLD, nullptr, tid, MmScaled{1.0f / sqrtf((float)D)});
    kr_.store(ks, QLD, nullptr, tid, MmScaled{1.f});
  }
  __syncthreads();
  // scores of the wave's 16 tokens against the tokens of the column tiles up to its own
  lc_f32x4 sc[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) sc[i] = lc_f32x4{0.f, 0.f, 0.f, 0.f};
  const float* qrow = qs + (16 * wave + r) * QLD + g;
#pragma unroll 4
  for (int k4 = 0; k4 < DP / 4; ++k4) {
    const float a = qrow[4 * k4];
#pragma unroll
    for (int ct = 0; ct < 4; ++ct)
      if (ct <= wave) sc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, ks[(16 * ct + r) * QLD + 4 * k4 + g], sc[ct], 0, 0, 0);
  }
  __syncthreads();                        // every wave has read the keys: their place takes the weighted scores and the values
  float* ps = ks;
  vr_.store_turned(vs, tid);
#pragma unroll
  for (int ct = 0; ct < 4; ++ct)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * g + i, s = 16 * ct + r;
      ps[t * PLD + s] = ct <= wave && s <= t ? sc[ct][i] * expf((float)(as[s] - Ms[t])) : 0.f;
    }
  __syncthreads();
  lc_f32x4 acc[4], far[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) acc[i] = far[i] = lc_f32x4{0.f, 0.f, 0.f, 0.f};
  const float* prow = ps + (16 * wave + r) * PLD + g;
  for (int k4 = 0; k4 < 4 * (wave + 1); ++k4) {
    const float a = prow[4 * k4];
    const float* vr = vs + (4 * k4 + g) * LC_V + r;
#pragma unroll
    for (int cv = 0; cv < 4; ++cv) acc[cv] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, vr[16 * (cv ^ g)], acc[cv], 0, 0, 0);
  }
  // what the state before the chunk adds: q S, each row times e^(m - M_t)
#pragma unroll
  for (int k4 = 0; k4 < AHEAD; ++k4) {
    const float a = qrow[4 * k4];
#pragma unroll
    for (int cv = 0; cv < 4; ++cv) far[cv] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, sv[k4][cv], far[cv], 0, 0, 0);
  }
#pragma unroll 8
  for (int k4 = AHEAD; k4 < DP / 4; ++k4) {
    const float a = qrow[4 * k4];
    const int d = 4 * k4 + g;
#pragma unroll
    for (int cv = 0; cv < 4; ++cv) {
      const float bv = d < D && v0 + 16 * cv + r < V ? sb[(size_t)d * V + 16 * cv] : 0.f;
      far[cv] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, bv, far[cv], 0, 0, 0);
    }
  }
#pragma unroll
  for (int cv = 0; cv < 4; ++cv) {
    const int v = v0 + 16 * cv + r;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * g + i;
      if (t < nc && v < V)
        num[((size_t)(t0 + c * LC_T + t) * H + h) * V + v] = fmaf(coef[t], far[cv][i], acc[cv][i]);
    }
  }
  if (blockIdx.x != 0) return;
  // n . q of a token by four neighbouring threads: the weighted scores' sum and the part of the n before the chunk
  {
    const int t = tid / 4, part = tid % 4;
    float s = 0.f, f = 0.f;
    for (int x = part; x <= t; x += 4) s += ps[t * PLD + x];
    const float* nb = chunk + (size_t)H * D * V + (size_t)h * D;
    for (int d = part; d < D; d += 4) f = fmaf(qs[t * QLD + d], nb[d], f);
    float nq = fmaf(coef[t], f, s);
    nq += __shfl_xor(nq, 1, TQ_WAVE);
    nq += __shfl_xor(nq, 2, TQ_WAVE);
    if (part == 0 && t < nc) den[(size_t)(t0 + c * LC_T + t) * H + h] = fmaxf(fabsf(nq), expf(-mt[t])) + MM_EPS;
  }
  if (tid == 0 && (c + 1) * LC_T >= n)
    state[(size_t)slots[b] * state_stride + (size_t)H * D * V + (size_t)H * D + h] = mt[nc - 1];
}

template <int ND, bool VEC>
static int mm_chunked_launch(const float* P, int64_t ldp, const float* bias, float cap, const int* cu_seqlens, const int* slots,
                             float* state, int64_t state_stride, int B, int NC, int max_chunks, int H, int D, int V,
                             float* scratch, double* scal, float* num, float* den, hipStream_t st) {
  constexpr int DP = 16 * ND, KLD = DP + (80 - DP % 64) % 64, QLD = DP + 4,
                KROWS = QLD > LC_T + 4 + LC_V ? QLD : LC_T + 4 + LC_V;
  const size_t sh_state = ((size_t)LC_T * KLD + (size_t)LC_T * LC_VLD + LC_T) * sizeof(float);
  const size_t sh_out = ((size_t)LC_T * QLD + (size_t)LC_T * KROWS + 6 * LC_T) * sizeof(float);
  if (sh_state > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)mm_chunk_state_kernel<ND, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)sh_state);
  if (sh_out > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)mm_chunk_out_kernel<ND, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)sh_out);
  const dim3 grid((V + LC_V - 1) / LC_V, H, B * NC);
  hipLaunchKernelGGL((mm_chunk_state_kernel<ND, VEC>), grid, dim3(256), sh_state, st, P, ldp, bias, cap, cu_seqlens, NC,
                     max_chunks, H, D, V, scratch, scal);
  hipLaunchKernelGGL(mm_chunk_prefix_kernel, dim3((D * V + D + 255) / 256, H, B), dim3(256), 0, st, cu_seqlens, slots, state,
                     state_stride, max_chunks, H, D, V, scratch, scal);
  hipLaunchKernelGGL((mm_chunk_out_kernel<ND, VEC>), grid, dim3(256), sh_out, st, P, ldp, bias, cap, cu_seqlens, slots, state,
                     state_stride, NC, max_chunks, H, D, V, scratch, scal, num, den);
  TQ_LAUNCH_CHECK();
  return 0;
}

// As tq_mm_scan, for steps with long runs, m included: max_new is the longest run's number of tokens, scratch holds max_chunks *
// H (D V + D) floats and scal max_chunks * 3 H doubles with max_chunks >= sum_b ceil(n_b / 64) (T / 64 + B is always enough).
TQ_API int tq_mm_chunked(const float* P, int64_t ldp, const float* bias, float cap, const int* cu_seqlens, const int* slots,
                         float* state, int64_t state_stride, int B, int H, int D, int V, int max_new, float* scratch,
                         double* scal, int max_chunks, float* num, float* den, hipStream_t st) {
  if (B <= 0 || max_new <= 0) return 0;
  if (H < 1 || D < 1 || V < 1 || ldp < (int64_t)2 * H * (D + V + 1) || state_stride < (int64_t)H * ((int64_t)D * V + D + 1) ||
      !(cap > 0.f) || !bias || !scratch || !scal || max_chunks < 1 || !num || !den)
    return TQ_ERR_BAD_ARG;
  const int NC = (max_new + LC_T - 1) / LC_T;
  if (D > 256 || H > 65535 || (int64_t)B * NC > 65535 || (int64_t)D * V + D > (int64_t)256 * 65535) return TQ_ERR_UNSUPPORTED;
  // whole rows of four floats: every row of every head starts at a multiple of 16 bytes
  const bool vec = D % 4 == 0 && V % 4 == 0 && ldp % 4 == 0 && (uintptr_t)P % 16 == 0;
#define TQ_MC(NDV)                                                                                                        \
  return vec ? mm_chunked_launch<NDV, true>(P, ldp, bias, cap, cu_seqlens, slots, state, state_stride, B, NC, max_chunks, H, \
                                            D, V, scratch, scal, num, den, st)                                            \
             : mm_chunked_launch<NDV, false>(P, ldp, bias, cap, cu_seqlens, slots, state, state_stride, B, NC, max_chunks, H, \
                                             D, V, scratch, scal, num, den, st)
  if (D <= 16) TQ_MC(1);
  if (D <= 32) TQ_MC(2);
  if (D <= 64) TQ_MC(4);
  if (D <= 128) TQ_MC(8);
  TQ_MC(16);
#undef TQ_MC
}

// ------------------------------------------------------------------------------------------ norm, weight and gate
// out[t][h V + v] = o / sqrt(mean_v(o^2) + eps) * w[h V + v] * sigmoid(g[t][h V + v]) with o = num / den, in the activation type; the
// gate's row of token t at gate + t * ldg.  A workgroup a token, a wave to every fourth head.  mrow (null: none) holds the
// running maxima that mm_scan found: those of every run's last token (the next token of the step belongs to another slot)
// go into the rows of state.
template <class W>
__global__ __launch_bounds__(256) void mm_out_kernel(const float* __restrict__ num, const float* __restrict__ den,
                                                     const float* __restrict__ gate, int64_t ldg, const W* __restrict__ w,
                                                     float eps, act_t* __restrict__ out, int64_t ldo, int T, int H, int V,
                                                     const float* __restrict__ mrow, const int* __restrict__ slot_of_token,
                                                     float* __restrict__ state_m, int64_t state_stride) {
  const int t = blockIdx.x, wave = threadIdx.x / TQ_WAVE, lane = threadIdx.x % TQ_WAVE;
  for (int h = wave; h < H; h += 4) {
    const float* row = num + ((size_t)t * H + h) * V;
    const float d = 1.0f / den[(size_t)t * H + h];
    float ss = 0.f;
    for (int i = lane; i < V; i += TQ_WAVE) {
      const float o = row[i] * d;
      ss = fmaf(o, o, ss);
    }
    ss = wave_sum(ss);
    const float rs = d * (1.0f / sqrtf(ss / (float)V + eps));
    const float* g = gate + (size_t)t * ldg + (size_t)h * V;
    for (int i = lane; i < V; i += TQ_WAVE)
      out[(size_t)t * ldo + h * V + i] = from_f32<act_t>(row[i] * rs * to_f32(w[h * V + i]) * (1.0f / (1.0f + expf(-g[i]))));
  }
  if (mrow && (t == T - 1 || slot_of_token[t + 1] != slot_of_token[t]))
    for (int h = threadIdx.x; h < H; h += 256)
      state_m[(size_t)slot_of_token[t] * state_stride + h] = mrow[(size_t)t * H + h];
}

// ldo: numbers between the rows of two tokens in out.  state (with mrow): the rows of all slots, whose last H floats are m at offset m_offset.
TQ_API int tq_mm_out(const float* num, const float* den, const float* gate, int64_t ldg, const void* w, int wtype, float eps,
                     void* out, int64_t ldo, int T, int H, int V, const float* mrow, const int* slot_of_token, float* state,
                     int64_t state_stride, int64_t m_offset, hipStream_t st) {
  if (T <= 0) return 0;
  if (H < 1 || V < 1 || ldg < (int64_t)H * V || ldo < (int64_t)H * V || !w || !gate || !den) return TQ_ERR_BAD_ARG;
  if (mrow && (!slot_of_token || !state || m_offset < 0 || state_stride < m_offset + H)) return TQ_ERR_BAD_ARG;
  TQ_DISPATCH_W(wtype, {
    hipLaunchKernelGGL(mm_out_kernel<W>, dim3(T), dim3(256), 0, st, num, den, gate, ldg, (const W*)w, eps, (act_t*)out, ldo, T, H, V,
                       mrow, slot_of_token, state ? state + m_offset : state, state_stride);
  });
  TQ_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------------------------------ decoding
// One token per sequence (token b of the step is sequence b's): grid (H, B), block 1024.  Threads stand as RG groups of key
// channels by V / 4 groups of value channels; a thread takes every RG-th key channel of its four value channels, MM_HOLD of
// them at a time in registers.
// A mixer beside the memory may have its queries, keys and values of the same step laid out by the same launch: one more
// workgroup per token (blockIdx.x == H) turns nothing, takes the token's row of qkv (nh query heads, nkv key heads, nkv value
// heads of hd numbers), puts the queries into q_out and keys and values (these transposed) into the page that holds the token's
// position, as rope_kv_write does without a rotation.
#define MM_HOLD 4
struct MmKvWrite {
  const float* qkv;             // rows ldp apart, like P's (null: nothing to write)
  const int* positions;
  const int* block_table;
  int bt_stride;
  act_t *q_out, *k_pool, *v_pool;
  int page_size;
  int64_t page_stride;
  int nh, nkv, hd;
};

__device__ __forceinline__ void mm_write_kv(const MmKvWrite& k, int64_t ldp, int slot, int b) {
  const float* row = k.qkv + (size_t)b * ldp;
  const int pos = k.positions[b];
  const int64_t page = k.block_table[(size_t)slot * k.bt_stride + pos / k.page_size];
  const int r = pos % k.page_size, nq = k.nh * k.hd, nk = k.nkv * k.hd;
  act_t* kp = k.k_pool + page * k.page_stride + (size_t)r * k.hd;
  act_t* vp = k.v_pool + page * k.page_stride + r;
  for (int i = threadIdx.x; i < nq + 2 * nk; i += blockDim.x) {
    const act_t x = from_f32<act_t>(row[i]);
    if (i < nq) {
      k.q_out[(size_t)b * nq + i] = x;
    } else if (i < nq + nk) {
      const int h = (i - nq) / k.hd, d = (i - nq) % k.hd;
      kp[(size_t)h * k.page_size * k.hd + d] = x;
    } else {
      const int h = (i - nq - nk) / k.hd, d = (i - nq - nk) % k.hd;
      vp[((size_t)h * k.hd + d) * k.page_size] = x;
    }
  }
}

template <class W>
__global__ __launch_bounds__(1024) void mm_decode_kernel(const float* __restrict__ P, int64_t ldp,
                                                         const float* __restrict__ bias, float cap,
                                                         const int* __restrict__ slots, float* __restrict__ state,
                                                         int64_t state_stride, int H, int D, int V,
                                                         const W* __restrict__ w, float eps, act_t* __restrict__ out,
                                                         int64_t ldo, MmKvWrite kvw) {
  if ((int)blockIdx.x == H) {
    mm_write_kv(kvw, ldp, slots[blockIdx.y], blockIdx.y);
    return;
  }
  __shared__ float qs[1024], ks[1024], red[16];
  __shared__ __align__(16) float part[4096];       // [RG][V]
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int CG = V / 4, RG = 1024 / CG;
  const int cg = tid % CG, rg = tid / CG;
  const float* row = P + (size_t)b * ldp;
  float* srow = state + (size_t)slots[b] * state_stride;
  float* S0 = srow + (size_t)h * D * V + 4 * cg;
  float* n0 = srow + (size_t)H * D * V + (size_t)h * D;
  float* m0 = srow + (size_t)H * D * V + (size_t)H * D + h;
  float4 S[MM_HOLD];
#pragma unroll
  for (int u = 0; u < MM_HOLD; ++u) {
    const int d = rg + u * RG;
    S[u] = rg < RG && d < D ? *reinterpret_cast<const float4*>(S0 + (size_t)d * V) : float4{0.f, 0.f, 0.f, 0.f};
  }
  const float4 val = rg < RG ? *reinterpret_cast<const float4*>(row + (size_t)2 * H * D + (size_t)h * V + 4 * cg)
                             : float4{0.f, 0.f, 0.f, 0.f};
  const float* g0 = row + (size_t)2 * H * (D + V) + h;
  const float m = *m0;
  float gi, gf;
  mm_gates(g0[0], g0[H], bias[h], bias[H + h], cap, gi, gf);
  const float mn = fmaxf(gf + m, gi), keep = expf(gf + m - mn), add = expf(gi - mn);
  const float scale = 1.0f / sqrtf((float)D);
  float nq = 0.f;
  for (int d = tid; d < D; d += 1024) {
    const float q = scale * row[(size_t)h * D + d], k = row[(size_t)H * D + (size_t)h * D + d];
    qs[d] = q;
    ks[d] = add * k;
    const float n = fmaf(keep, n0[d], add * k);
    n0[d] = n;
    nq = fmaf(n, q, nq);
  }
  nq = block_sum(nq, red);       // (its barriers also stand between the rows' stores and their use, and before m is written)
  if (tid == 0) *m0 = mn;
  const float inv = 1.0f / (fmaxf(fabsf(nq), expf(-mn)) + MM_EPS);
  float4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int d0 = rg; rg < RG && d0 < D; d0 += MM_HOLD * RG) {
    if (d0 != rg) {
#pragma unroll
      for (int u = 0; u < MM_HOLD; ++u) {
        const int d = d0 + u * RG;
        if (d < D) S[u] = *reinterpret_cast<const float4*>(S0 + (size_t)d * V);
      }
    }
#pragma unroll
    for (int u = 0; u < MM_HOLD; ++u) {
      const int d = d0 + u * RG;
      if (d < D) {
        const float k = ks[d], q = qs[d];
        float4 s = S[u];
        s.x = fmaf(keep, s.x, k * val.x);
        s.y = fmaf(keep, s.y, k * val.y);
        s.z = fmaf(keep, s.z, k * val.z);
        s.w = fmaf(keep, s.w, k * val.w);
        *reinterpret_cast<float4*>(S0 + (size_t)d * V) = s;
        acc.x = fmaf(s.x, q, acc.x);
        acc.y = fmaf(s.y, q, acc.y);
        acc.z = fmaf(s.z, q, acc.z);
        acc.w = fmaf(s.w, q, acc.w);
      }
    }
  }
  if (rg < RG) *reinterpret_cast<float4*>(part + (size_t)rg * V + 4 * cg) = acc;
  __syncthreads();
  float o = 0.f;
  if (tid < V) {
#pragma unroll 8
    for (int x = 0; x < RG; ++x) o += part[(size_t)x * V + tid];
    o *= inv;
  }
  const float ss = block_sum(o * o, red);
  if (tid < V) {
    const float g = row[(size_t)2 * H * D + (size_t)H * V + (size_t)h * V + tid];
    out[(size_t)b * ldo + h * V + tid] =
        from_f32<act_t>(o * (1.0f / sqrtf(ss / (float)V + eps)) * to_f32(w[h * V + tid]) * (1.0f / (1.0f + expf(-g))));
  }
}

// A decode step's memory in one launch: the recurrence on every sequence's row of state (m included), norm, weight and gate;
// out [B][H V] in the activation type, rows ldo apart.  Takes value widths that are multiples of 4 up to 1,024 and key widths
// up to 1,024, with rows of P and of the state that start at multiples of 16 bytes.  qkv (null: none), positions [B],
// block_table [slots][bt_stride], q_out [B][nh hd], k_pool, v_pool (the layer's offset added): MmKvWrite.
TQ_API int tq_mm_decode(const float* P, int64_t ldp, const float* bias, float cap, const int* slots, float* state,
                        int64_t state_stride, int B, int H, int D, int V, const void* w, int wtype, float eps, void* out,
                        int64_t ldo, const float* qkv, const int* positions, const int* block_table, int bt_stride, void* q_out,
                        void* k_pool, void* v_pool, int page_size, int64_t page_stride, int nh, int nkv, int hd,
                        hipStream_t st) {
  if (B <= 0) return 0;
  if (H < 1 || D < 1 || V < 1 || ldp < (int64_t)2 * H * (D + V + 1) || state_stride < (int64_t)H * ((int64_t)D * V + D + 1) ||
      !(cap > 0.f) || !bias || !w || ldo < (int64_t)H * V)
    return TQ_ERR_BAD_ARG;
  if (qkv && (!positions || !block_table || bt_stride < 1 || !q_out || !k_pool || !v_pool || page_size < 1 || nh < 1 || nkv < 1 ||
              hd < 1 || ldp < (int64_t)(nh + 2 * nkv) * hd))
    return TQ_ERR_BAD_ARG;
  if (V % 4 || V > 1024 || D > 1024 || H > 65534 || B > 65535 || ldp % 4 || state_stride % 4 || (2 * H * D) % 4 ||
      (uintptr_t)P % 16 || (uintptr_t)state % 16)
    return TQ_ERR_UNSUPPORTED;
  const MmKvWrite kvw{qkv, positions, block_table, bt_stride, (act_t*)q_out, (act_t*)k_pool, (act_t*)v_pool, page_size,
                      page_stride, nh, nkv, hd};
  TQ_DISPATCH_W(wtype, {
    hipLaunchKernelGGL(mm_decode_kernel<W>, dim3(H + (qkv ? 1 : 0), B), dim3(1024), 0, st, P, ldp, bias, cap, slots, state,
                       state_stride, H, D, V, (const W*)w, eps, (act_t*)out, ldo, kvw);
  });
  TQ_LAUNCH_CHECK();
  return 0;
}
