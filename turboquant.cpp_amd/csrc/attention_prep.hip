// What stands between the product of a layer's input and its attention, for two kinds of attention that the launches in
// elementwise.hip do not know:
//   row_norm_kv_write   query and key norm over a token's whole projection (all heads together), rotation, cache write; the
//                       values may be the keys as they were projected
//   diff_prep_kv_write  two maps a head (differential attention): a norm per head and map, a factor on the queries that grows
//                       with the position, cache write with both maps of a key head side by side in one row
// and behind such an attention
//   diff_combine        the two maps' outputs made one, normed per head, gated.
// Float arithmetic; queries, keys and values leave in the activation type.
#include "value_tiles.h"

// ------------------------------------------------------------------------------------------ one norm over all heads
// qkv[t] (row stride ld): nh query heads, nkv key heads, then nkv value heads of hd each, the values at head first_value
// (nh: the keys' own rows).  q / sqrt(sum(q^2) / q_dim + eps) * wq over all of q's numbers, k alike (wq, wk [heads * hd], zeros
// where heads are laid out wider than they are), then the rotation as in rope_kv_write.  A wave takes a head at a time; the
// sums over the whole rows are made by every workgroup for itself.
template <class W>
__global__ __launch_bounds__(256) void row_norm_kv_write_kernel(
    const float* __restrict__ qkv, int64_t ld, const int* __restrict__ positions, const int* __restrict__ seq_of_token,
    const int* __restrict__ block_table, int bt_stride, const float* __restrict__ inv_freq, int pairing, int rot, float amp,
    const W* __restrict__ wq, const W* __restrict__ wk, float eps, int q_dim, int k_dim, int first_value,
    act_t* __restrict__ q_out, act_t* __restrict__ k_pool, act_t* __restrict__ v_pool, int page_size, int64_t page_stride, int nh,
    int nkv, int hd, int write_kv, int spb) {
  __shared__ float red[256 / TQ_WAVE];
  const int t = blockIdx.x;
  const int wave = threadIdx.x / TQ_WAVE, lane = threadIdx.x % TQ_WAVE;
  const int heads = nh + 2 * nkv;
  const int b0 = blockIdx.y * spb, b1 = min(b0 + spb, heads);
  const int s0 = b0 + wave;
  const float* src_t = qkv + (size_t)t * ld;
  float rs[2] = {1.f, 1.f};
#pragma unroll
  for (int part = 0; part < 2; ++part) {
    // (the same for the whole workgroup: whether it has heads of this kind)
    const bool needs = part == 0 ? b0 < nh : (b1 > nh && b0 < nh + nkv && write_kv);
    if (!needs) continue;
    const float* row = src_t + (part ? (size_t)nh * hd : 0);
    const int n = (part ? nkv : nh) * hd;
    float ss = 0.f;
    if (hd % 4 == 0 && ld % 4 == 0) {
#pragma unroll 4
      for (int i = threadIdx.x * 4; i < n; i += 1024) {
        const f32x4 v = load4f(row + i);
        ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
      }
    } else {
      for (int i = threadIdx.x; i < n; i += 256) ss = fmaf(row[i], row[i], ss);
    }
    rs[part] = 1.0f / sqrtf(block_sum(ss, red) / (float)(part ? k_dim : q_dim) + eps);
  }
  if (s0 >= b1) return;
  const int pos = positions[t];
  act_t* q_t = q_out + (size_t)t * nh * hd;
  act_t *k_t = nullptr, *v_t = nullptr;
  if (write_kv && b1 > nh) {
    const int page = block_table[(size_t)seq_of_token[t] * bt_stride + pos / page_size];
    const int row = pos % page_size;
    k_t = k_pool + (size_t)page * page_stride + (size_t)row * hd;
    v_t = v_pool + (size_t)page * page_stride + row;
  }
  const int rot_end = write_kv ? min(b1, nh + nkv) : min(b1, nh);
  const size_t kv_head_stride = (size_t)page_size * hd;
  const int half = rot / 2;
  for (int i = lane; i < half; i += TQ_WAVE) {
    float sn, cs;
    sincosf((float)pos * inv_freq[i], &sn, &cs);
    sn *= amp;
    cs *= amp;
    const int ia = pairing == 0 ? i : 2 * i;
    const int ib = pairing == 0 ? i + half : 2 * i + 1;
    for (int s = s0; s < rot_end; s += 4) {
      const float* src = src_t + (size_t)s * hd;
      const W* w = s < nh ? wq + (size_t)s * hd : wk + (size_t)(s - nh) * hd;
      const float r = s < nh ? rs[0] : rs[1];
      act_t* dst = s < nh ? q_t + (size_t)s * hd : k_t + (size_t)(s - nh) * kv_head_stride;
      const float a = src[ia] * r * to_f32(w[ia]), b = src[ib] * r * to_f32(w[ib]);
      dst[ia] = from_f32<act_t>(a * cs - b * sn);
      dst[ib] = from_f32<act_t>(a * sn + b * cs);
    }
  }
  for (int s = s0; s < rot_end; s += 4) {      // dimensions from rot on pass through
    const float* src = src_t + (size_t)s * hd;
    const W* w = s < nh ? wq + (size_t)s * hd : wk + (size_t)(s - nh) * hd;
    const float r = s < nh ? rs[0] : rs[1];
    act_t* dst = s < nh ? q_t + (size_t)s * hd : k_t + (size_t)(s - nh) * kv_head_stride;
    for (int i = rot + lane; i < hd; i += TQ_WAVE) dst[i] = from_f32<act_t>(src[i] * r * to_f32(w[i]));
  }
  if (write_kv != 1) return;
  for (int s = s0; s < b1; s += 4) {           // values lie transposed, [hd][row]
    if (s < nh + nkv) continue;
    const float* src = src_t + (size_t)(first_value + s - nh - nkv) * hd;
    act_t* col = v_t + (size_t)(s - nh - nkv) * kv_head_stride;
    for (int i = lane; i < hd; i += TQ_WAVE) col[(size_t)i * page_size] = from_f32<act_t>(src[i]);
  }
}

// How many of `heads` heads a workgroup takes: few tokens a head to a wave, many tokens all heads of a token together.
static int heads_per_workgroup(int T, int heads) {
  int spb = 4;
  while (spb < heads && (int64_t)T * ((heads + spb - 1) / spb) > 4096) spb *= 2;
  return spb;
}

// Arguments as tq_rope_kv_write_ex's, with the norms' weights, the numbers q and k really have (q_dim, k_dim) and the head of
// the row that holds the first value head.  nkv may be 0 with write_kv 0 (queries for another layer's keys).
TQ_API int tq_row_norm_kv_write(const float* qkv, int64_t ld, const int* positions, const int* seq_of_token,
                                const int* block_table, int bt_stride, const float* inv_freq, int pairing, int rot, float amp,
                                const void* wq, const void* wk, int wtype, float eps, int q_dim, int k_dim, int first_value,
                                void* q_out, void* k_pool, void* v_pool, int page_size, int64_t page_stride, int T, int nh, int nkv,
                                int hd, int write_kv, const int* cu_seqlens, const int* slots, const int* start, int B,
                                int max_new, hipStream_t st) {
  if (T <= 0) return 0;
  if (rot < 0 || rot % 2 != 0 || rot > hd || (pairing != 0 && pairing != 1) || nh < 1 || nkv < 0 || hd < 1) return TQ_ERR_BAD_ARG;
  if (!wq || q_dim < 1 || (write_kv && (!wk || k_dim < 1 || !k_pool || !v_pool || nkv < 1 || first_value < nh))) return TQ_ERR_BAD_ARG;
  if (ld < (int64_t)(nh + (write_kv ? nkv : 0)) * hd || (write_kv && ld < (int64_t)(first_value + nkv) * hd)) return TQ_ERR_BAD_ARG;
  const bool tiles = write_kv && value_tiles_fit(cu_seqlens, slots, start, B, nkv, hd, max_new, page_size);
  if (tiles) write_kv = 2;
  const int heads = write_kv == 1 ? nh + 2 * nkv : write_kv ? nh + nkv : nh;
  const int spb = heads_per_workgroup(T, heads);
  if ((heads + spb - 1) / spb > 65535) return TQ_ERR_UNSUPPORTED;
  TQ_DISPATCH_W(wtype, {
    hipLaunchKernelGGL(row_norm_kv_write_kernel<W>, dim3(T, (heads + spb - 1) / spb), dim3(256), 0, st, qkv, ld, positions,
                       seq_of_token, block_table, bt_stride, inv_freq, pairing, rot, amp, (const W*)wq, (const W*)wk, eps, q_dim,
                       k_dim, first_value, (act_t*)q_out, (act_t*)k_pool, (act_t*)v_pool, page_size, page_stride, nh, nkv, hd,
                       write_kv, spb);
  });
  TQ_LAUNCH_CHECK();
  if (tiles) {
    launch_value_tiles<0>(qkv, nullptr, cu_seqlens, slots, start, block_table, bt_stride, v_pool, page_size, page_stride, first_value,
                          nkv, hd, ld, B, max_new, st);
    TQ_LAUNCH_CHECK();
  }
  return 0;
}

// ------------------------------------------------------------------------------------------ two maps a head
// qkv[t] (row stride ld): nh query heads, nkv key heads, nkv value heads of hd = 2 half each; a query or key head is its map 1
// then its map 2, of half numbers each (zeros behind the norm_dim that they have).  Every map: x / sqrt(sum(x^2) / norm_dim +
// eps) * w, w = wq or wk [half], queries also times 1 + coef ln(floor((pos + 1) / every) + 1) (coef 0: not).  Keys and values
// go to the pages as rows of hd.  expand 0: q_out [T][nh][hd], both maps side by side; 1: q_out [T][2 nh][hd], each map alone
// with zeros in the other's place, so that its scores against the pages' rows are that map's.  A wave takes a head at a time.
template <class W>
__global__ __launch_bounds__(256) void diff_prep_kv_write_kernel(
    const float* __restrict__ qkv, int64_t ld, const int* __restrict__ positions, const int* __restrict__ seq_of_token,
    const int* __restrict__ block_table, int bt_stride, const W* __restrict__ wq, const W* __restrict__ wk, float eps, int norm_dim,
    float coef, float every, act_t* __restrict__ q_out, act_t* __restrict__ k_pool, act_t* __restrict__ v_pool, int page_size,
    int64_t page_stride, int nh, int nkv, int hd, int write_kv, int expand, int spb) {
  const int t = blockIdx.x;
  const int wave = threadIdx.x / TQ_WAVE, lane = threadIdx.x % TQ_WAVE;
  const int heads = nh + 2 * nkv, half = hd / 2;
  const int s0 = blockIdx.y * spb + wave, s1 = min(blockIdx.y * spb + spb, heads);
  if (s0 >= s1) return;
  const int pos = positions[t];
  const float* src_t = qkv + (size_t)t * ld;
  act_t *k_t = nullptr, *v_t = nullptr;
  if (write_kv && s1 > nh) {
    const int page = block_table[(size_t)seq_of_token[t] * bt_stride + pos / page_size];
    const int row = pos % page_size;
    k_t = k_pool + (size_t)page * page_stride + (size_t)row * hd;
    v_t = v_pool + (size_t)page * page_stride + row;
  }
  const size_t kv_head_stride = (size_t)page_size * hd;
  const float temp = coef != 0.f ? 1.0f + coef * logf(floorf((float)(pos + 1) / every) + 1.0f) : 1.0f;
  const int norm_end = write_kv ? min(s1, nh + nkv) : min(s1, nh);
  for (int s = s0; s < norm_end; s += 4) {
    const float* src = src_t + (size_t)s * hd;
    const W* w = s < nh ? wq : wk;
    float ss[2] = {0.f, 0.f};
    for (int i = lane; i < half; i += TQ_WAVE) {
      ss[0] = fmaf(src[i], src[i], ss[0]);
      ss[1] = fmaf(src[half + i], src[half + i], ss[1]);
    }
    const float f = s < nh ? temp : 1.0f;
    const float r0 = 1.0f / sqrtf(wave_sum(ss[0]) / (float)norm_dim + eps);
    const float r1 = 1.0f / sqrtf(wave_sum(ss[1]) / (float)norm_dim + eps);
    act_t* dst = s >= nh ? k_t + (size_t)(s - nh) * kv_head_stride
                         : q_out + (expand ? ((size_t)t * 2 * nh + 2 * s) * hd : ((size_t)t * nh + s) * hd);
    const bool two = s < nh && expand;
    for (int i = lane; i < half; i += TQ_WAVE) {
      const float wt = to_f32(w[i]);
      dst[i] = from_f32<act_t>(src[i] * r0 * wt * f);
      dst[(two ? hd : 0) + half + i] = from_f32<act_t>(src[half + i] * r1 * wt * f);
      if (two) dst[half + i] = dst[hd + i] = from_f32<act_t>(0.f);
    }
  }
  if (write_kv != 1) return;
  for (int s = s0; s < s1; s += 4) {
    if (s < nh + nkv) continue;
    const float* src = src_t + (size_t)s * hd;
    act_t* col = v_t + (size_t)(s - nh - nkv) * kv_head_stride;
    for (int i = lane; i < hd; i += TQ_WAVE) col[(size_t)i * page_size] = from_f32<act_t>(src[i]);
  }
}

TQ_API int tq_diff_prep_kv_write(const float* qkv, int64_t ld, const int* positions, const int* seq_of_token,
                                 const int* block_table, int bt_stride, const void* wq, const void* wk, int wtype, float eps,
                                 int norm_dim, float coef, float every, void* q_out, void* k_pool, void* v_pool, int page_size,
                                 int64_t page_stride, int T, int nh, int nkv, int hd, int write_kv, int expand,
                                 const int* cu_seqlens, const int* slots, const int* start, int B, int max_new, hipStream_t st) {
  if (T <= 0) return 0;
  if (hd < 2 || hd % 2 != 0 || nh < 1 || nkv < 0 || norm_dim < 1 || norm_dim > hd / 2 || !wq || (coef != 0.f && !(every > 0.f)))
    return TQ_ERR_BAD_ARG;
  if (write_kv && (!wk || !k_pool || !v_pool || nkv < 1)) return TQ_ERR_BAD_ARG;
  if (ld < (int64_t)(nh + (write_kv ? 2 * nkv : 0)) * hd) return TQ_ERR_BAD_ARG;
  const bool tiles = write_kv && value_tiles_fit(cu_seqlens, slots, start, B, nkv, hd, max_new, page_size);
  if (tiles) write_kv = 2;
  const int heads = write_kv == 1 ? nh + 2 * nkv : write_kv ? nh + nkv : nh;
  const int spb = heads_per_workgroup(T, heads);
  if ((heads + spb - 1) / spb > 65535) return TQ_ERR_UNSUPPORTED;
  TQ_DISPATCH_W(wtype, {
    hipLaunchKernelGGL(diff_prep_kv_write_kernel<W>, dim3(T, (heads + spb - 1) / spb), dim3(256), 0, st, qkv, ld, positions,
                       seq_of_token, block_table, bt_stride, (const W*)wq, (const W*)wk, eps, norm_dim, coef, every, (act_t*)q_out,
                       (act_t*)k_pool, (act_t*)v_pool, page_size, page_stride, nh, nkv, hd, write_kv, expand, spb);
  });
  TQ_LAUNCH_CHECK();
  if (tiles) {
    launch_value_tiles<0>(qkv, nullptr, cu_seqlens, slots, start, block_table, bt_stride, v_pool, page_size, page_stride, nh + nkv,
                          nkv, hd, ld, B, max_new, st);
    TQ_LAUNCH_CHECK();
  }
  return 0;
}

// o [T][2 nh][hd]: the two maps' outputs of every head.  out[t][h] = r / sqrt(sum(r^2) / vd + eps) * post * sigmoid(gate) with
// r = o[t][2 h] - lambda o[t][2 h + 1] (the values' first vd numbers; zeros behind them); gate: float rows [T][ld_gate] of nh hd
// numbers, or null.  A wave a head.
__global__ __launch_bounds__(256) void diff_combine_kernel(const act_t* __restrict__ o, float lambda, float eps, int vd, float post,
                                                           const float* __restrict__ gate, int64_t ld_gate, act_t* __restrict__ out,
                                                           int nh, int hd, int64_t items) {
  const int64_t item = (int64_t)blockIdx.x * 4 + threadIdx.x / TQ_WAVE;
  if (item >= items) return;
  const int lane = threadIdx.x % TQ_WAVE;
  const int64_t t = item / nh;
  const int h = (int)(item % nh);
  const act_t *a1 = o + (size_t)item * 2 * hd, *a2 = a1 + hd;
  float ss = 0.f;
  for (int i = lane; i < hd; i += TQ_WAVE) {
    const float r = to_f32(a1[i]) - lambda * to_f32(a2[i]);
    ss = fmaf(r, r, ss);
  }
  const float f = post / sqrtf(wave_sum(ss) / (float)vd + eps);
  const float* g = gate ? gate + (size_t)t * ld_gate + (size_t)h * hd : nullptr;
  for (int i = lane; i < hd; i += TQ_WAVE) {
    float r = (to_f32(a1[i]) - lambda * to_f32(a2[i])) * f;
    if (g) r /= 1.0f + expf(-g[i]);
    out[(size_t)item * hd + i] = from_f32<act_t>(r);
  }
}

TQ_API int tq_diff_combine(const void* o, float lambda, float eps, int vd, float post, const float* gate, int64_t ld_gate, void* out,
                           int T, int nh, int hd, hipStream_t st) {
  if (T <= 0) return 0;
  if (nh < 1 || hd < 1 || vd < 1 || vd > hd || (gate && ld_gate < (int64_t)nh * hd)) return TQ_ERR_BAD_ARG;
  const int64_t items = (int64_t)T * nh;
  if ((items + 3) / 4 > 0x7fffffff) return TQ_ERR_UNSUPPORTED;
  hipLaunchKernelGGL(diff_combine_kernel, dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, (const act_t*)o, lambda, eps, vd, post,
                     gate, ld_gate, (act_t*)out, nh, hd, items);
  TQ_LAUNCH_CHECK();
  return 0;
}
