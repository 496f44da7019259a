// Selective state spaces in their dual form (the Mamba-2 mixer), over per-sequence state of fixed size.
//
// Projections P [T][ldp] (float): z (H V) | x (H V) | B (G N) | C (G N) | dt (H).  x, B and C pass a causal convolution over
// time, one filter and a bias per channel, and silu; dt <- softplus(dt + dt_bias).  Per head h, which reads group h / (H / G)
// of B and C, with a state S [N][V] that starts at zero, token by token:
//   S <- exp(-exp(A_log_h) dt) S + dt B x^T ;  y = S^T C + D_h x
// and then, over all heads of a token, y silu(z) divided by its root mean square in `parts` equal parts, times a weight.
// Everything here is float arithmetic on both libraries (sums of decays over a chunk in double); the products around it are
// the library's.
//
// A sequence's row of state (float): S as [H][N][V], then for every channel of x, B, C its last taps - 1 inputs, oldest first.
//
//   ssd_prep     per token: convolution (its first inputs from the sequence's state), silu, step sizes
//   ssd_scan     short runs: the recurrence over a run's tokens in order, the state in registers
//   ssd_chunked  long runs in chunks of LC_T tokens on the matrix cores in float: see below
//   ssd_decode   one token per sequence: convolution, step size, recurrence and read-out in one launch
//   ssd_out      per token: gate, norm, weight, into the activation type; per sequence: the convolution's new state
#include "linear_chunks.h"
#include "value_tiles.h"

struct SsdDims {
  int H, V, N, G, taps;
};
__host__ __device__ __forceinline__ int sd_inner(const SsdDims& d) { return d.H * d.V; }
__host__ __device__ __forceinline__ int sd_channels(const SsdDims& d) { return d.H * d.V + 2 * d.G * d.N; }
__host__ __device__ __forceinline__ int sd_dt(const SsdDims& d) { return d.H * d.V + sd_channels(d); }      // where dt starts in P

static int sd_check(const SsdDims& d, int64_t ldp, int64_t state_stride) {
  if (d.H < 1 || d.V < 1 || d.N < 1 || d.G < 1 || d.taps < 1 || d.H % d.G != 0) return TQ_ERR_BAD_ARG;
  if (ldp < (int64_t)sd_dt(d) + d.H) return TQ_ERR_BAD_ARG;
  if (state_stride < (int64_t)d.H * d.N * d.V + (int64_t)sd_channels(d) * (d.taps - 1)) return TQ_ERR_BAD_ARG;
  return d.taps > 64 ? TQ_ERR_UNSUPPORTED : 0;
}

__device__ __forceinline__ float sd_silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float sd_softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// ------------------------------------------------------------------------------------------ per token
// The c-th token of its run has `before` = min(c, taps - 1) tokens of the run right before it (runs lie one behind the other,
// so they are the tokens with its slot); what it needs from further back is the state's.
// grid (ceil(T / SD_TOKENS), ceil(C / channels of a workgroup)), block 256.  E: channels of a thread (4: rows and channels
// start at multiples of 16 bytes).  TAPS: a window of that many inputs per channel stays in registers (fewer taps: zeros in
// front), 0: any number of taps, every input read anew.
#define SD_TOKENS 8
template <int E, int TAPS>
__global__ __launch_bounds__(256) void ssd_prep_kernel(const float* __restrict__ P, int64_t ldp,
                                                       const int* __restrict__ slot_of_token, const float* __restrict__ state,
                                                       int64_t state_stride, const float* __restrict__ conv_w,
                                                       const float* __restrict__ conv_b, const float* __restrict__ dt_bias,
                                                       SsdDims d, float* __restrict__ xbc, float* __restrict__ dt, int T) {
  const int C = sd_channels(d), K = d.taps, H = d.H;
  const int t0 = blockIdx.x * SD_TOKENS, t1 = min(t0 + SD_TOKENS, T);
  if (blockIdx.y == 0) {
    const int at = sd_dt(d);
    for (int i = threadIdx.x; i < (t1 - t0) * H; i += 256) {
      const int t = t0 + i / H, h = i % H;
      dt[(size_t)t * H + h] = sd_softplus(P[(size_t)t * ldp + at + h] + dt_bias[h]);
    }
  }
  const int c = (blockIdx.y * 256 + threadIdx.x) * E;
  if (c >= C) return;
  const float* col = P + sd_inner(d) + c;
  const int64_t hist0 = (int64_t)H * d.N * d.V + (int64_t)c * (K - 1);
  float bias[E];
#pragma unroll
  for (int e = 0; e < E; ++e) bias[e] = conv_b[c + e];
  auto tokens_before = [&](int t) {
    const int slot = slot_of_token[t];
    int n = 0;
    while (n < K - 1 && t - n - 1 >= 0 && slot_of_token[t - n - 1] == slot) ++n;
    return n;
  };
  // the input `back` tokens before token t, which has `before` tokens of its run behind it
  auto input = [&](int t, int back, int before, float (&in)[E]) {
    if (back <= before) {
      if constexpr (E == 4) {
        const f32x4 v = load4f(col + (size_t)(t - back) * ldp);
        in[0] = v.x, in[1] = v.y, in[2] = v.z, in[3] = v.w;
      } else {
        in[0] = col[(size_t)(t - back) * ldp];
      }
    } else {
      const float* h = state + (size_t)slot_of_token[t] * state_stride + hist0 + (K - 1) - (back - before);
#pragma unroll
      for (int e = 0; e < E; ++e) in[e] = h[(size_t)e * (K - 1)];
    }
  };
  if constexpr (TAPS > 0) {
    float w[TAPS][E], win[TAPS][E];      // w[k], win[k]: the tap and the input k tokens back
#pragma unroll
    for (int k = 0; k < TAPS; ++k)
#pragma unroll
      for (int e = 0; e < E; ++e) {
        w[k][e] = k < K ? conv_w[(size_t)(c + e) * K + K - 1 - k] : 0.f;
        win[k][e] = 0.f;
      }
    for (int t = t0; t < t1; ++t) {
      if (t == t0 || slot_of_token[t] != slot_of_token[t - 1]) {
        const int before = tokens_before(t);
#pragma unroll
        for (int k = 1; k < TAPS; ++k)
          if (k < K) input(t, k, before, win[k]);
      } else {
#pragma unroll
        for (int k = TAPS - 1; k >= 1; --k)
#pragma unroll
          for (int e = 0; e < E; ++e) win[k][e] = win[k - 1][e];
      }
      input(t, 0, 0, win[0]);
      float y[E];
#pragma unroll
      for (int e = 0; e < E; ++e) {
        float s = bias[e];
#pragma unroll
        for (int k = TAPS - 1; k >= 0; --k) s = fmaf(w[k][e], win[k][e], s);
        y[e] = sd_silu(s);
      }
      float* to = xbc + (size_t)t * C + c;
      if constexpr (E == 4) store4(to, f32x4{y[0], y[1], y[2], y[3]});
      else to[0] = y[0];
    }
  } else {
    for (int t = t0; t < t1; ++t) {
      const int before = tokens_before(t);
      float s[E];
#pragma unroll
      for (int e = 0; e < E; ++e) s[e] = bias[e];
      for (int k = K - 1; k >= 0; --k) {
        float in[E];
        input(t, k, before, in);
#pragma unroll
        for (int e = 0; e < E; ++e) s[e] = fmaf(conv_w[(size_t)(c + e) * K + K - 1 - k], in[e], s[e]);
      }
#pragma unroll
      for (int e = 0; e < E; ++e) xbc[(size_t)t * C + c + e] = sd_silu(s[e]);
    }
  }
}

// xbc [T][H V + 2 G N] and dt [T][H] (float) from the step's projections; nothing of the state is written.
TQ_API int tq_ssd_prep(const float* P, int64_t ldp, const int* slot_of_token, const float* state, int64_t state_stride,
                       const float* conv_w, const float* conv_b, const float* dt_bias, int H, int V, int N, int G, int taps,
                       float* xbc, float* dt, int T, hipStream_t st) {
  if (T <= 0) return 0;
  const SsdDims d{H, V, N, G, taps};
  const int rc = sd_check(d, ldp, state_stride);
  if (rc) return rc;
  const int C = sd_channels(d);
  const bool vec = C % 4 == 0 && ldp % 4 == 0 && sd_inner(d) % 4 == 0 && (uintptr_t)P % 16 == 0 && (uintptr_t)xbc % 16 == 0;
  const int per = vec ? 1024 : 256;
  const dim3 grid((T + SD_TOKENS - 1) / SD_TOKENS, (C + per - 1) / per);
  if (grid.y > 65535) return TQ_ERR_UNSUPPORTED;
#define TQ_SD_PREP(E, TAPS)                                                                                                     \
  hipLaunchKernelGGL((ssd_prep_kernel<E, TAPS>), grid, dim3(256), 0, st, P, ldp, slot_of_token, state, state_stride, conv_w, conv_b, \
                     dt_bias, d, xbc, dt, T)
  if (taps <= 4) {
    if (vec) TQ_SD_PREP(4, 4);
    else TQ_SD_PREP(1, 4);
  } else {
    if (vec) TQ_SD_PREP(4, 0);
    else TQ_SD_PREP(1, 0);
  }
#undef TQ_SD_PREP
  TQ_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------------------------------ short runs
// grid (ceil(V / VB), H, B), block 256; L = lanes per value channel (a power of two, L * SD_ROWS >= N), VB = 256 / L.
#define SD_ROWS 16        // state channels of a value channel that one lane keeps
#define SD_SEG 20         // floats between the rows of two lanes in LDS
#define SD_STAGED(L) ((L) > 16 ? 4 : 16)       // tokens staged at a time
template <int L>
__global__ __launch_bounds__(256) void ssd_scan_kernel(const float* __restrict__ xbc, const float* __restrict__ dt,
                                                       const float* __restrict__ a_log, const float* __restrict__ Dh,
                                                       const int* __restrict__ cu_seqlens, const int* __restrict__ slots,
                                                       float* __restrict__ state, int64_t state_stride, SsdDims d,
                                                       float* __restrict__ y) {
  constexpr int VB = 256 / L, CH = SD_STAGED(L);
  __shared__ float cs[CH][L * SD_SEG], bs[CH][L * SD_SEG], xs[CH][VB], keep_s[CH], dt_s[CH];
  const int H = d.H, V = d.V, N = d.N, C = sd_channels(d);
  const int b = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * VB, grp = h / (H / d.G);
  const int tid = threadIdx.x, vc = tid / L, j = tid % L;
  const int v = v0 + vc;
  const bool live = v < V;
  const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
  if (n <= 0) return;
  float* srow = state + (size_t)slots[b] * state_stride + (size_t)h * N * V;
  const float rate = -expf(a_log[h]), skip = Dh[h];
  float S[SD_ROWS];
#pragma unroll
  for (int r = 0; r < SD_ROWS; ++r) {
    const int i = j * SD_ROWS + r;
    S[r] = live && i < N ? srow[(size_t)i * V + v] : 0.f;
  }
  const float* x0 = xbc + (size_t)h * V + v0;
  const float* B0 = xbc + sd_inner(d) + (size_t)grp * N;
  const float* C0 = B0 + (size_t)d.G * N;
  for (int c0 = 0; c0 < n; c0 += CH) {
    const int nc = min(CH, n - c0);
    __syncthreads();
    for (int idx = tid; idx < nc * L * SD_ROWS; idx += 256) {
      const int c = idx / (L * SD_ROWS), i = idx % (L * SD_ROWS);
      const size_t row = (size_t)(t0 + c0 + c) * C;
      const int at = (i / SD_ROWS) * SD_SEG + i % SD_ROWS;
      cs[c][at] = i < N ? C0[row + i] : 0.f;
      bs[c][at] = i < N ? B0[row + i] : 0.f;
    }
    for (int idx = tid; idx < nc * VB; idx += 256) {
      const int c = idx / VB, i = idx % VB;
      xs[c][i] = v0 + i < V ? x0[(size_t)(t0 + c0 + c) * C + i] : 0.f;
    }
    if (tid < nc) {
      const float s = dt[(size_t)(t0 + c0 + tid) * H + h];
      dt_s[tid] = s;
      keep_s[tid] = expf(rate * s);
    }
    __syncthreads();
    for (int c = 0; c < nc; ++c) {
      const float keep = keep_s[c], x = xs[c][vc], val = dt_s[c] * x;
      const float* br = &bs[c][j * SD_SEG];
      const float* cr = &cs[c][j * SD_SEG];
      float acc = 0.f;
#pragma unroll
      for (int r = 0; r < SD_ROWS; ++r) {
        S[r] = fmaf(keep, S[r], br[r] * val);
        acc = fmaf(S[r], cr[r], acc);
      }
#pragma unroll
      for (int off = L / 2; off > 0; off >>= 1) acc += __shfl_xor(acc, off, TQ_WAVE);
      if (j == 0 && live) y[((size_t)(t0 + c0 + c) * H + h) * V + v] = fmaf(skip, x, acc);
    }
  }
  if (live) {
#pragma unroll
    for (int r = 0; r < SD_ROWS; ++r) {
      const int i = j * SD_ROWS + r;
      if (i < N) srow[(size_t)i * V + v] = S[r];
    }
  }
}

// xbc, dt: what tq_ssd_prep left; a_log, D [H]; cu_seqlens [B + 1], slots [B]: the tokens as one run per sequence; y [T][H V].
TQ_API int tq_ssd_scan(const float* xbc, const float* dt, const float* a_log, const float* D, const int* cu_seqlens,
                       const int* slots, float* state, int64_t state_stride, int H, int V, int N, int G, int taps, int B, float* y,
                       hipStream_t st) {
  if (B <= 0) return 0;
  const SsdDims d{H, V, N, G, taps};
  const int rc = sd_check(d, (int64_t)sd_dt(d) + H, state_stride);
  if (rc) return rc;
  if (N > 64 * SD_ROWS || H > 65535 || B > 65535) return TQ_ERR_UNSUPPORTED;
  int L = 1;
  while (L * SD_ROWS < N) L *= 2;
#define TQ_SD_SCAN(LV)                                                                                                        \
  hipLaunchKernelGGL(ssd_scan_kernel<LV>, dim3((V + 256 / LV - 1) / (256 / LV), H, B), dim3(256), 0, st, xbc, dt, a_log, D,   \
                     cu_seqlens, slots, state, state_stride, d, y)
  switch (L) {
    case 1: TQ_SD_SCAN(1); break;
    case 2: TQ_SD_SCAN(2); break;
    case 4: TQ_SD_SCAN(4); break;
    case 8: TQ_SD_SCAN(8); break;
    case 16: TQ_SD_SCAN(16); break;
    case 32: TQ_SD_SCAN(32); break;
    default: TQ_SD_SCAN(64); break;
  }
#undef TQ_SD_SCAN
  TQ_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------------------------------ long runs, in chunks
// With a_t = -exp(A_log) dt_t <= 0, F_t the sum of a over a chunk's tokens up to t, S the state before the chunk:
//   y_t    = sum_{s <= t} e^(F_t - F_s) dt_s (C_t . B_s) x_s + e^(F_t) S^T C_t + D x_t
//   state' = e^(F_n) S + sum_s e^(F_n - F_s) dt_s B_s x_s^T
// No exponent is positive.  Three launches: every chunk's own sum (chunks side by side); the states before the chunks, per
// element over a sequence's chunks in order (the sequence's row of state is read first and written last); every chunk's
// read-outs.  F is kept in double: a chunk's F may reach some hundreds, of which differences are taken.  A workgroup takes
// `hb` heads of one group one after the other: they share B and C, and the products C B^T of a chunk.
// scratch (float): per chunk H N V; tot (float): per chunk and head e^(F_n).
#define SD_HEADS 4       // most heads of a workgroup: one wave each works out their F

struct SdSame {
  __device__ __forceinline__ float operator()(float x) const { return x; }
};

__device__ __forceinline__ double sd_scan_sum(double x, int lane) {      // inclusive, over a wave's lanes
#pragma unroll
  for (int o = 1; o < TQ_WAVE; o <<= 1) {
    const double up = __shfl_up(x, o, TQ_WAVE);
    if (lane >= o) x += up;
  }
  return x;
}

// grid (ceil(V / LC_V), H / hb, B * NC), block 256: a chunk's own sum, a wave to 16 value channels.
template <int ND, bool VEC>
__global__ __launch_bounds__(256) void ssd_chunk_state_kernel(const float* __restrict__ xbc, const float* __restrict__ dt,
                                                              const float* __restrict__ a_log, const int* __restrict__ cu_seqlens,
                                                              int NC, int cap, SsdDims d, int hb, float* __restrict__ scratch,
                                                              float* __restrict__ tot) {
  extern __shared__ __align__(16) float sd_lds[];
  constexpr int DP = 16 * ND, KLD = DP + (80 - DP % 64) % 64;
  float* ks = sd_lds;                    // [LC_T][KLD]
  float* vs = ks + LC_T * KLD;           // [LC_T][LC_VLD], each token's values times its weight
  float* wt = vs + LC_T * LC_VLD;        // [SD_HEADS][LC_T]
  const int H = d.H, V = d.V, N = d.N, C = sd_channels(d);
  const int b = blockIdx.z / NC, c = blockIdx.z % NC, h0 = blockIdx.y * hb, v0 = blockIdx.x * LC_V, grp = h0 / (H / d.G);
  const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
  if (c * LC_T >= n) return;
  const int gi = lc_chunk_base(cu_seqlens, b) + c;
  if (gi >= cap) return;
  const int nc = min(LC_T, n - c * LC_T), tid = threadIdx.x;
  const int wave = tid / 64, lane = tid % 64, g = lane / 16, r = lane % 16;
  const float* row0 = xbc + (size_t)(t0 + c * LC_T) * C;
  LcRows<LC_V, VEC> vr_;
  {
    LcRows<DP, VEC> kr_;
    kr_.fetch(row0 + sd_inner(d) + (size_t)grp * N, C, nc, N, tid);
    vr_.fetch(row0 + (size_t)h0 * V + v0, C, nc, V - v0, tid);
    if (wave < hb) {
      const float s = lane < nc ? dt[(size_t)(t0 + c * LC_T + lane) * H + h0 + wave] : 0.f;
      const double F = sd_scan_sum((double)(-expf(a_log[h0 + wave]) * s), lane);
      const double Fn = __shfl(F, TQ_WAVE - 1, TQ_WAVE);
      wt[wave * LC_T + lane] = s * expf((float)(Fn - F));
      if (blockIdx.x == 0 && lane == 0) tot[(size_t)gi * H + h0 + wave] = expf((float)Fn);
    }
    kr_.store(ks, KLD, nullptr, tid, SdSame());
  }
  __syncthreads();
  for (int u = 0; u < hb; ++u) {
    vr_.store(vs, LC_VLD, wt + u * LC_T, tid, SdSame());
    __syncthreads();
    if (u + 1 < hb) vr_.fetch(row0 + (size_t)(h0 + u + 1) * V + v0, C, nc, V - v0, tid);
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
    const int v = v0 + 16 * wave + r;
    if (v < V) {
      float* out = scratch + ((size_t)gi * H + h0 + u) * N * V + v;
#pragma unroll
      for (int rt = 0; rt < ND; ++rt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int k = 16 * rt + 4 * g + i;
          if (k < N) out[(size_t)k * V] = acc[rt][i];
        }
    }
    __syncthreads();
  }
}

// grid (ceil(N V / 256), H, B), block 256: every chunk's own sum becomes the state before it, in place; the row of state is
// advanced.
#define SD_AHEAD 16       // chunks whose sums are asked for before the first of them is replaced
__global__ __launch_bounds__(256) void ssd_chunk_prefix_kernel(const int* __restrict__ cu_seqlens, const int* __restrict__ slots,
                                                               float* __restrict__ state, int64_t state_stride, int cap, SsdDims d,
                                                               float* __restrict__ scratch, const float* __restrict__ tot) {
  const int b = blockIdx.z, h = blockIdx.y, H = d.H, NV = d.N * d.V;
  const int e = blockIdx.x * 256 + threadIdx.x;
  const int n = cu_seqlens[b + 1] - cu_seqlens[b];
  if (n <= 0 || e >= NV) return;
  const int base = lc_chunk_base(cu_seqlens, b), chunks = (n + LC_T - 1) / LC_T;
  if (base + chunks > cap) return;
  float* srow = state + (size_t)slots[b] * state_stride + (size_t)h * NV + e;
  float carry = *srow;
  float* at = scratch + ((size_t)base * H + h) * NV + e;
  const float* keep = tot + (size_t)base * H + h;
  for (int c0 = 0; c0 < chunks; c0 += SD_AHEAD) {
    float own[SD_AHEAD], k[SD_AHEAD];
#pragma unroll
    for (int u = 0; u < SD_AHEAD; ++u) {
      const int c = min(c0 + u, chunks - 1);
      own[u] = at[(size_t)c * H * NV];
      k[u] = keep[(size_t)c * H];
    }
#pragma unroll
    for (int u = 0; u < SD_AHEAD; ++u)
      if (c0 + u < chunks) {
        at[(size_t)(c0 + u) * H * NV] = carry;
        carry = fmaf(k[u], carry, own[u]);
      }
  }
  *srow = carry;
}

// grid (ceil(V / LC_V), H / hb, B * NC), block 256: a chunk's read-outs for LC_V value channels.  (The
// values wait in registers until B has been read and take its place in LDS: with states of up to 128 channels two workgroups
// fit a compute unit.)
template <int ND, bool VEC>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(ND > 8 ? 1 : 2))) void ssd_chunk_out_kernel(
    const float* __restrict__ xbc, const float* __restrict__ dt, const float* __restrict__ a_log, const float* __restrict__ Dh,
    const int* __restrict__ cu_seqlens, int NC, int cap, SsdDims d, int hb, const float* __restrict__ scratch,
    float* __restrict__ y) {
  extern __shared__ __align__(16) float sd_lds[];
  constexpr int DP = 16 * ND, QLD = DP + 4, PLD = LC_T + 4;
  double* Fs = reinterpret_cast<double*>(sd_lds);          // [SD_HEADS][LC_T]
  float* dts = reinterpret_cast<float*>(Fs + SD_HEADS * LC_T);      // [SD_HEADS][LC_T]
  float* qs = dts + SD_HEADS * LC_T;     // [LC_T][QLD]: C
  float* ks = qs + LC_T * QLD;           // [LC_T][QLD]: B; later the weighted scores [LC_T][PLD]
  float* vs = ks + LC_T * PLD;           // and the values [LC_T][LC_V] behind them
  const int H = d.H, V = d.V, N = d.N, C = sd_channels(d);
  const int b = blockIdx.z / NC, c = blockIdx.z % NC, h0 = blockIdx.y * hb, v0 = blockIdx.x * LC_V, grp = h0 / (H / d.G);
  const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
  if (c * LC_T >= n) return;
  const int gi = lc_chunk_base(cu_seqlens, b) + c;
  if (gi >= cap) return;
  const int nc = min(LC_T, n - c * LC_T), tid = threadIdx.x;
  const int wave = tid / 64, lane = tid % 64, g = lane / 16, r = lane % 16;
  const float* row0 = xbc + (size_t)(t0 + c * LC_T) * C;
  LcRows<LC_V, VEC> vr_;
  {
    LcRows<DP, VEC> qr_, kr_;
    kr_.fetch(row0 + sd_inner(d) + (size_t)grp * N, C, nc, N, tid);
    qr_.fetch(row0 + sd_inner(d) + (size_t)(d.G + grp) * N, C, nc, N, tid);
    vr_.fetch(row0 + (size_t)h0 * V + v0, C, nc, V - v0, tid);
    if (wave < hb) {
      const float s = lane < nc ? dt[(size_t)(t0 + c * LC_T + lane) * H + h0 + wave] : 0.f;
      Fs[wave * LC_T + lane] = sd_scan_sum((double)(-expf(a_log[h0 + wave]) * s), lane);
      dts[wave * LC_T + lane] = s;
    }
    qr_.store(qs, QLD, nullptr, tid, SdSame());
    kr_.store(ks, QLD, nullptr, tid, SdSame());
  }
  __syncthreads();
  // C B^T: the wave's 16 tokens against the tokens of the column tiles up to its own, the same for every head of the group
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
  float* ps = ks;
  // From here on a wave takes 16 value channels of all the chunk's tokens, so that it reads its columns of the state once.
  // (Loads are unconditional, from addresses within the state: rows beyond N meet zeros of C, columns beyond V are not stored.)
  const int v = v0 + 16 * wave + r, vl = min(v, V - 1);
  const float* sb = scratch + ((size_t)gi * H + h0) * N * V + vl;
  constexpr int AHEAD = DP / 4 > 32 ? 32 : DP / 4;
  for (int u = 0; u < hb; ++u) {
    const int h = h0 + u;
    const double* F = Fs + u * LC_T;
    const float* step = dts + u * LC_T;
    float sv[AHEAD];
#pragma unroll
    for (int k4 = 0; k4 < AHEAD; ++k4) sv[k4] = sb[(size_t)min(4 * k4 + g, N - 1) * V];
    __syncthreads();                      // every wave has read B, or the scores and values of the head before
    vr_.store_turned(vs, tid);
#pragma unroll
    for (int ct = 0; ct < 4; ++ct)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * wave + 4 * g + i, s = 16 * ct + r;
        ps[t * PLD + s] = ct <= wave && s <= t ? sc[ct][i] * (expf((float)(F[t] - F[s])) * step[s]) : 0.f;
      }
    __syncthreads();
    if (u + 1 < hb) vr_.fetch(row0 + (size_t)(h + 1) * V + v0, C, nc, V - v0, tid);
    lc_f32x4 acc[4], far[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = far[i] = lc_f32x4{0.f, 0.f, 0.f, 0.f};
    // the chunk's own tokens: a tile of 16 of them reaches the tiles up to its own
#pragma unroll
    for (int ct = 0; ct < 4; ++ct)
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const int k4 = 4 * ct + k;
        const float bv = vs[(4 * k4 + g) * LC_V + ((16 * wave + r) ^ (16 * g))];
#pragma unroll
        for (int tt = 0; tt < 4; ++tt)
          if (tt >= ct) acc[tt] = __builtin_amdgcn_mfma_f32_16x16x4f32(ps[(16 * tt + r) * PLD + 4 * k4 + g], bv, acc[tt], 0, 0, 0);
      }
    // what the state before the chunk adds: S^T C, each row times e^(F_t)
    const float* qr = qs + r * QLD + g;
#pragma unroll
    for (int k4 = 0; k4 < AHEAD; ++k4)
#pragma unroll
      for (int tt = 0; tt < 4; ++tt)
        far[tt] = __builtin_amdgcn_mfma_f32_16x16x4f32(qr[16 * tt * QLD + 4 * k4], sv[k4], far[tt], 0, 0, 0);
#pragma unroll 8
    for (int k4 = AHEAD; k4 < DP / 4; ++k4) {
      const float bv = sb[(size_t)min(4 * k4 + g, N - 1) * V];
#pragma unroll
      for (int tt = 0; tt < 4; ++tt)
        far[tt] = __builtin_amdgcn_mfma_f32_16x16x4f32(qr[16 * tt * QLD + 4 * k4], bv, far[tt], 0, 0, 0);
    }
    const float skip = Dh[h];
    if (v < V)
#pragma unroll
      for (int tt = 0; tt < 4; ++tt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 16 * tt + 4 * g + i;
          if (t < nc) {
            const float x = vs[t * LC_V + ((16 * wave + r) ^ (16 * (t & 3)))];
            y[((size_t)(t0 + c * LC_T + t) * H + h) * V + v] = fmaf(skip, x, fmaf(expf((float)F[t]), far[tt][i], acc[tt][i]));
          }
        }
    sb += (size_t)N * V;
  }
}

template <int ND, bool VEC>
static int ssd_chunked_launch(const float* xbc, const float* dt, const float* a_log, const float* D, const int* cu_seqlens,
                              const int* slots, float* state, int64_t state_stride, const SsdDims& d, int B, int NC, int cap, int hb,
                              float* scratch, float* tot, float* y, hipStream_t st) {
  constexpr int DP = 16 * ND, KLD = DP + (80 - DP % 64) % 64, QLD = DP + 4, PLD = LC_T + 4;
  constexpr int KROWS = QLD > PLD + LC_V ? QLD : PLD + LC_V;
  const size_t sh_state = ((size_t)LC_T * KLD + (size_t)LC_T * LC_VLD + SD_HEADS * LC_T) * sizeof(float);
  const size_t sh_out = ((size_t)LC_T * QLD + (size_t)LC_T * KROWS + 3 * SD_HEADS * LC_T) * sizeof(float);
  if (sh_state > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)ssd_chunk_state_kernel<ND, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)sh_state);
  if (sh_out > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)ssd_chunk_out_kernel<ND, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)sh_out);
  const dim3 grid((d.V + LC_V - 1) / LC_V, d.H / hb, B * NC);
  hipLaunchKernelGGL((ssd_chunk_state_kernel<ND, VEC>), grid, dim3(256), sh_state, st, xbc, dt, a_log, cu_seqlens, NC, cap, d, hb,
                     scratch, tot);
  hipLaunchKernelGGL(ssd_chunk_prefix_kernel, dim3((d.N * d.V + 255) / 256, d.H, B), dim3(256), 0, st, cu_seqlens, slots, state,
                     state_stride, cap, d, scratch, tot);
  hipLaunchKernelGGL((ssd_chunk_out_kernel<ND, VEC>), grid, dim3(256), sh_out, st, xbc, dt, a_log, D, cu_seqlens, NC, cap, d, hb,
                     scratch, y);
  TQ_LAUNCH_CHECK();
  return 0;
}

// As tq_ssd_scan, for steps with long runs: max_new is the longest run's number of tokens; scratch holds chunks * H N V floats
// and tot chunks * H with chunks >= sum_b ceil(n_b / 64) (T / 64 + B is always enough).
TQ_API int tq_ssd_chunked(const float* xbc, const float* dt, const float* a_log, const float* D, const int* cu_seqlens,
                          const int* slots, float* state, int64_t state_stride, int H, int V, int N, int G, int taps, int B,
                          int max_new, float* scratch, float* tot, int chunks, float* y, hipStream_t st) {
  if (B <= 0 || max_new <= 0) return 0;
  const SsdDims d{H, V, N, G, taps};
  const int rc = sd_check(d, (int64_t)sd_dt(d) + H, state_stride);
  if (rc) return rc;
  if (!scratch || !tot || chunks < 1) return TQ_ERR_BAD_ARG;
  const int NC = (max_new + LC_T - 1) / LC_T;
  if (N > 256 || H > 65535 || (int64_t)B * NC > 65535 || (int64_t)N * V > (int64_t)256 * 65535) return TQ_ERR_UNSUPPORTED;
  const int C = sd_channels(d);
  const bool vec = N % 4 == 0 && V % 4 == 0 && C % 4 == 0 && (uintptr_t)xbc % 16 == 0;
  // heads of a group to a workgroup, as long as the chip still has two workgroups to a compute unit
  int hb = 1;
  const int64_t wgs = (int64_t)((V + LC_V - 1) / LC_V) * H * B * NC;
  while (hb * 2 <= SD_HEADS && (H / G) % (hb * 2) == 0 && wgs / (hb * 2) >= 512) hb *= 2;
#define TQ_SD(NDV)                                                                                                              \
  return vec ? ssd_chunked_launch<NDV, true>(xbc, dt, a_log, D, cu_seqlens, slots, state, state_stride, d, B, NC, chunks, hb,   \
                                             scratch, tot, y, st)                                                               \
             : ssd_chunked_launch<NDV, false>(xbc, dt, a_log, D, cu_seqlens, slots, state, state_stride, d, B, NC, chunks, hb,  \
                                              scratch, tot, y, st)
  if (N <= 16) TQ_SD(1);
  if (N <= 32) TQ_SD(2);
  if (N <= 64) TQ_SD(4);
  if (N <= 128) TQ_SD(8);
  TQ_SD(16);
#undef TQ_SD
}

// ------------------------------------------------------------------------------------------ one token per sequence
// grid (ceil(V / VB), H, B), block 256: convolution, step size, recurrence and read-out for VB = LANES * E value channels of a
// head.  The first rows of the state are asked for before anything else.  The convolution's inputs in the state are read here
// and moved on by ssd_out, which runs behind: several heads read those of B and C.
template <int LANES, int E>
__global__ __launch_bounds__(256) void ssd_decode_kernel(const float* __restrict__ P, int64_t ldp, const int* __restrict__ slots,
                                                         float* __restrict__ state, int64_t state_stride,
                                                         const float* __restrict__ conv_w, const float* __restrict__ conv_b,
                                                         const float* __restrict__ dt_bias, const float* __restrict__ a_log,
                                                         const float* __restrict__ Dh, SsdDims d, float* __restrict__ y) {
  constexpr int VB = LANES * E, RG = 256 / LANES, AHEAD = 8;
  extern __shared__ __align__(16) float sd_lds[];
  float* bs = sd_lds;                    // [N] dt B
  float* cs = bs + d.N;                  // [N]
  float* xs = cs + d.N;                  // [VB]
  float* red = xs + VB;                  // [RG][VB]
  const int H = d.H, V = d.V, N = d.N, K = d.taps;
  const int b = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * VB, grp = h / (H / d.G);
  const int tid = threadIdx.x, rg = tid / LANES, v = v0 + (tid % LANES) * E;
  float* row = state + (size_t)slots[b] * state_stride;
  float* S = row + (size_t)h * N * V + v;
  const bool live = v < V;
  float s[AHEAD][E];
  auto load = [&](int k, float (&to)[E]) {
    if constexpr (E == 4) {
      const f32x4 t = load4f(S + (size_t)k * V);
      to[0] = t.x, to[1] = t.y, to[2] = t.z, to[3] = t.w;
    } else {
      to[0] = S[(size_t)k * V];
    }
  };
#pragma unroll
  for (int u = 0; u < AHEAD; ++u)
    if (live && rg + u * RG < N) load(rg + u * RG, s[u]);
  const float* Pt = P + (size_t)b * ldp;
  const float* hist = row + (size_t)H * N * V;
  const float step = sd_softplus(Pt[sd_dt(d) + h] + dt_bias[h]);
  const float keep = expf(-expf(a_log[h]) * step);
  for (int i = tid; i < 2 * N + VB; i += 256) {
    const bool is_x = i >= 2 * N;
    const int c = is_x ? h * V + min(v0 + i - 2 * N, V - 1) : sd_inner(d) + (i < N ? grp * N + i : (d.G + grp) * N + i - N);
    float acc = conv_b[c];
    const float* w = conv_w + (size_t)c * K;
    const float* hc = hist + (size_t)c * (K - 1);
    for (int k = 0; k < K - 1; ++k) acc = fmaf(w[k], hc[k], acc);
    acc = sd_silu(fmaf(w[K - 1], Pt[sd_inner(d) + c], acc));
    sd_lds[i] = i < N ? step * acc : acc;      // (bs, cs and xs lie one behind the other)
  }
  __syncthreads();
  float acc[E], x[E];
#pragma unroll
  for (int e = 0; e < E; ++e) {
    acc[e] = 0.f;
    x[e] = xs[(tid % LANES) * E + e];
  }
  if (live) {
    for (int k0 = rg; k0 < N; k0 += AHEAD * RG) {
#pragma unroll
      for (int u = 0; u < AHEAD; ++u) {
        const int k = k0 + u * RG;
        if (k < N) {
          const float bk = bs[k], ck = cs[k];
#pragma unroll
          for (int e = 0; e < E; ++e) {
            s[u][e] = fmaf(keep, s[u][e], bk * x[e]);
            acc[e] = fmaf(s[u][e], ck, acc[e]);
          }
          if constexpr (E == 4) store4(S + (size_t)k * V, f32x4{s[u][0], s[u][1], s[u][2], s[u][3]});
          else S[(size_t)k * V] = s[u][0];
        }
      }
#pragma unroll
      for (int u = 0; u < AHEAD; ++u)
        if (k0 + (AHEAD + u) * RG < N) load(k0 + (AHEAD + u) * RG, s[u]);
    }
  }
#pragma unroll
  for (int e = 0; e < E; ++e) red[rg * VB + (tid % LANES) * E + e] = acc[e];
  __syncthreads();
  if (tid < VB && v0 + tid < V) {
    float o = 0.f;
#pragma unroll 8
    for (int i = 0; i < RG; ++i) o += red[i * VB + tid];
    y[((size_t)b * H + h) * V + v0 + tid] = fmaf(Dh[h], xs[tid], o);
  }
}

// P: the projections of one token per sequence [B][ldp]; y [B][H V].
TQ_API int tq_ssd_decode(const float* P, int64_t ldp, const int* slots, float* state, int64_t state_stride, const float* conv_w,
                         const float* conv_b, const float* dt_bias, const float* a_log, const float* D, int H, int V, int N, int G,
                         int taps, int B, float* y, hipStream_t st) {
  if (B <= 0) return 0;
  const SsdDims d{H, V, N, G, taps};
  const int rc = sd_check(d, ldp, state_stride);
  if (rc) return rc;
  if (H > 65535 || B > 65535 || N > 8192) return TQ_ERR_UNSUPPORTED;
  const bool vec = V % 4 == 0 && state_stride % 4 == 0 && (uintptr_t)state % 16 == 0;
#define TQ_SD_DECODE(LANES, E)                                                                                                  \
  do {                                                                                                                          \
    const int vb = LANES * E;                                                                                                   \
    const size_t shmem = ((size_t)2 * N + vb + (256 / LANES) * vb) * sizeof(float);                                             \
    if (shmem > 48 * 1024)                                                                                                      \
      (void)hipFuncSetAttribute((const void*)ssd_decode_kernel<LANES, E>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem); \
    hipLaunchKernelGGL((ssd_decode_kernel<LANES, E>), dim3((V + vb - 1) / vb, H, B), dim3(256), shmem, st, P, ldp, slots, state,  \
                       state_stride, conv_w, conv_b, dt_bias, a_log, D, d, y);                                                  \
  } while (0)
  if (vec && V <= 32) TQ_SD_DECODE(8, 4);
  else if (vec) TQ_SD_DECODE(16, 4);
  else TQ_SD_DECODE(64, 1);
#undef TQ_SD_DECODE
  TQ_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------------------------------ gate, norm, new inputs
// grid (T + B, Y), block 256.  Blocks 0 .. T - 1 of x: the token's parts dealt over y: y silu(z) divided by its root mean square
// over the part, times a weight per channel.  Blocks T ..: the convolution's state of one sequence, its channels dealt over y:
// its last taps - 1 inputs, those of this run and, where the run is shorter, the most recent of the old state before them.
template <class W, int E>
__global__ __launch_bounds__(256) void ssd_out_kernel(const float* __restrict__ y, const float* __restrict__ P, int64_t ldp,
                                                      const W* __restrict__ w, float eps, int parts,
                                                      const int* __restrict__ cu_seqlens, const int* __restrict__ slots,
                                                      float* __restrict__ state, int64_t state_stride, SsdDims d, int T,
                                                      act_t* __restrict__ out) {
  extern __shared__ __align__(16) float sd_lds[];
  __shared__ float red[256 / TQ_WAVE];
  const int inner = sd_inner(d), K = d.taps;
  if ((int)blockIdx.x >= T) {
    const int b = blockIdx.x - T, C = sd_channels(d);
    const int t0 = cu_seqlens[b], n = cu_seqlens[b + 1] - t0;
    if (n <= 0) return;
    float* hist = state + (size_t)slots[b] * state_stride + (size_t)d.H * d.N * d.V;
    for (int c = blockIdx.y * 256 + threadIdx.x; c < C; c += gridDim.y * 256)
      for (int j = 0; j < K - 1; ++j) {
        const int back = K - 2 - j;        // how many tokens before the run's last
        hist[(size_t)c * (K - 1) + j] = back < n ? P[(size_t)(t0 + n - 1 - back) * ldp + inner + c] : hist[(size_t)c * (K - 1) + j + n];
      }
    return;
  }
  const int t = blockIdx.x, width = inner / parts;
  for (int p = blockIdx.y; p < parts; p += gridDim.y) {
    const float* yr = y + (size_t)t * inner + (size_t)p * width;
    const float* zr = P + (size_t)t * ldp + (size_t)p * width;
    const W* wr = w + (size_t)p * width;
    act_t* to = out + (size_t)t * inner + (size_t)p * width;
    float ss = 0.f;
    for (int i = threadIdx.x * E; i < width; i += 256 * E) {
      if constexpr (E == 4) {
        const f32x4 z = load4f(zr + i);
        f32x4 v = load4f(yr + i);
        v = f32x4{v.x * sd_silu(z.x), v.y * sd_silu(z.y), v.z * sd_silu(z.z), v.w * sd_silu(z.w)};
        store4(sd_lds + i, v);
        ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
      } else {
        const float v = yr[i] * sd_silu(zr[i]);
        sd_lds[i] = v;
        ss = fmaf(v, v, ss);
      }
    }
    const float rs = 1.0f / sqrtf(block_sum(ss, red) / (float)width + eps);
    for (int i = threadIdx.x * E; i < width; i += 256 * E) {      // (a thread reads what it wrote itself)
      if constexpr (E == 4) store4(to + i, load4f(sd_lds + i) * rs * load4f(wr + i));
      else to[i] = from_f32<act_t>(sd_lds[i] * rs * to_f32(wr[i]));
    }
  }
}

TQ_API int tq_ssd_out(const float* y, const float* P, int64_t ldp, const void* w, int wtype, float eps, int parts,
                      const int* cu_seqlens, const int* slots, float* state, int64_t state_stride, int H, int V, int N, int G,
                      int taps, int T, int B, void* out, hipStream_t st) {
  if (T <= 0 || B <= 0) return 0;
  const SsdDims d{H, V, N, G, taps};
  const int rc = sd_check(d, ldp, state_stride);
  if (rc) return rc;
  const int inner = sd_inner(d);
  if (parts < 1 || inner % parts != 0 || !w) return TQ_ERR_BAD_ARG;
  const int width = inner / parts;
  const size_t shmem = (size_t)(width + 3) / 4 * 4 * sizeof(float);
  if (shmem > 150 * 1024) return TQ_ERR_UNSUPPORTED;
  const int channel_blocks = (sd_channels(d) + 255) / 256;
  int Y = parts > 1 || T <= 64 ? (parts > channel_blocks ? parts : channel_blocks) : 1;      // few tokens: channels dealt wide too
  if (parts > 1 && T > 64) Y = parts;
  Y = Y > 1024 ? 1024 : Y;
  const bool vec = width % 4 == 0 && ldp % 4 == 0 && (uintptr_t)P % 16 == 0 && (uintptr_t)y % 16 == 0;
  TQ_DISPATCH_W(wtype, {
    if (vec) {
      if (shmem > 48 * 1024)
        (void)hipFuncSetAttribute((const void*)ssd_out_kernel<W, 4>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem);
      hipLaunchKernelGGL((ssd_out_kernel<W, 4>), dim3(T + B, Y), dim3(256), shmem, st, y, P, ldp, (const W*)w, eps, parts, cu_seqlens,
                         slots, state, state_stride, d, T, (act_t*)out);
    } else {
      if (shmem > 48 * 1024)
        (void)hipFuncSetAttribute((const void*)ssd_out_kernel<W, 1>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem);
      hipLaunchKernelGGL((ssd_out_kernel<W, 1>), dim3(T + B, Y), dim3(256), shmem, st, y, P, ldp, (const W*)w, eps, parts, cu_seqlens,
                         slots, state, state_stride, d, T, (act_t*)out);
    }
  });
  TQ_LAUNCH_CHECK();
  return 0;
}
