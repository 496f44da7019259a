// Attention over the paged cache on the matrix cores (bfloat16 in, float softmax and sums).
//
// Formulas as in attention_generic.hip (/root/reference/src/engine/tq_transformer.c:1646-1654 window,
// :1675-1679 head mapping, :1908-1976 scores, softmax, value sum).  A wave works on 16 "columns" that
// share keys and values and runs over tiles of 64 cache positions (a page, or a quarter of one):
//
//   S^T = K Q^T     v_mfma_f32_16x16x32_bf16 with A = 16 keys x 32 of hd (16 bytes per lane straight from the
//                   page, keys lie [row][hd]) and B = the columns' queries, kept in registers.  The 16 rows of
//                   block jt are not 16 consecutive keys: row i is key 32 (jt / 2) + 8 (i / 4) + 4 (jt % 2) + i % 4,
//                   so that lane l, which holds rows 4 (l / 16) + v of every block for column l % 16, holds 8
//                   consecutive keys across the two blocks of a pair.
//   softmax         per column, that is per lane: maxima and sums over a lane's registers and over the four
//                   lanes l % 16 + 16 c; all in float, running maximum across tiles.
//   O^T += V^T P^T  A = 16 of hd x 32 keys (values lie transposed in the page, [hd][row], so a lane reads its 8
//                   consecutive keys of one dimension with 16 bytes) and B = the probabilities exactly as the
//                   lane already holds them.  No transpose through LDS anywhere.
//
// Two entry points share this: whole prompts (columns = 16 consecutive tokens of a sequence, one head; four
// waves per workgroup) and decoding (columns = the query heads that share one kv head, one token; the cache is
// split into runs of 1 or 3 tiles, one wave each, and a second kernel joins the runs in order).  Tiles start at
// multiples of 64 positions and runs at multiples of the run length, so the order of every sum depends only on
// the token's own position.
#include "common.h"
#include "score_mod.h"

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));
typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));

#define TILE 64
#define LOG2E 1.4426950408889634f
// Tiles per run when decoding a token at position p: short sequences are cut finer, so that a small batch still
// gives the chip hundreds of waves; a function of the token's own position only.  Measured with 16 kv heads: at
// position 8191, 3 tiles per run beat 4 by 15 % at 8 sequences and lose 2 to 4 % from 16 on, 2 lose 9 % and 1 loses
// 22 %; at positions 3000 and 4000, 1 tile per run beats 2 by 25 % and 9 % at 8 sequences (4 % and -2 % at 64).
__host__ __device__ __forceinline__ int tiles_per_run(int p) { return p >= 2 * 2048 ? 3 : 1; }
__host__ __device__ __forceinline__ int runs_at(int p) { return p / TILE / tiles_per_run(p) + 1; }
// Most runs that a token at a position below max_end can have.
static int most_runs(int max_end) {
  const int tiles = (max_end + 63) / 64;
  const int short_runs = tiles < 64 ? tiles : 64;          // below position 4096 no token has more than 64
  const int long_runs = (tiles + 2) / 3;
  return short_runs > long_runs ? short_runs : long_runs;
}

struct AttnArgs {
  const bf16_t* q;              // [T][nh][hd]
  const bf16_t* k_pool;         // layer's offset already added
  const bf16_t* v_pool;
  const int* block_table;
  int bt_stride;
  const int* cu_seqlens;        // [B + 1]
  const int* slots;             // [B]
  const int* start;             // [B] position of each sequence's first new token
  int page_size;
  int64_t page_stride;
  int nh, nkv, hd, window;
  float scale;
  bf16_t* out;                  // [T][nh][hd]
  float* partial;               // decoding: [B][nh][max_runs][hd + 2]
  int max_runs;
  ScoreMod mod;                 // what happens to a score before the softmax, and the chunks of positions (score_mod.h)
  const float* head_gate;       // null, or [T][ld_gate]: head h's output of token t is multiplied by sigmoid(head_gate[t][h])
  int64_t ld_gate;
  int64_t ldo;                  // numbers between the rows of two tokens in out (nh * hd, or more for columns of a wider matrix)
};

// Differential attention: a head attends with two maps, whose keys are the two halves of a key row, to the same values; what is
// left is r = a1 - lambda a2, divided by its root mean square over the values' vd numbers, times post, times sigmoid(gate).
struct DiffArgs {
  float lambda, eps, post;
  int vd;
  const float* gate;            // null, or [T][ld_gate] with nh * hd numbers a row
  int64_t ld_gate;
};

// What softmax_tile needs of the score's changes for the QG groups of columns a lane holds: the plain scale, the cap and
// each column's pair of the distance bias (a column is a token of one head in prompts, a head in decoding).
template <int QG, bool MOD>
struct ColMod {
  bool biased;
  float scale, cap;
  float r1[QG], r2[QG];
  bool sig;             // weights are sigmoids of score + pb, not normalised
  float pb[QG];
  int keep;             // first positions that stay visible whatever the window
};
template <int QG, bool MOD>
__device__ __forceinline__ ColMod<QG, MOD> col_mod(const AttnArgs& a, const int (&head)[QG]) {
  ColMod<QG, MOD> m;
  m.biased = MOD && a.mod.r1 != nullptr;
  m.scale = a.scale;
  m.cap = a.mod.cap;
#pragma unroll
  for (int g = 0; g < QG; ++g) {
    m.r1[g] = m.biased ? a.mod.r1[head[g]] : 0.f;
    m.r2[g] = m.biased ? a.mod.r2[head[g]] : 0.f;
  }
  m.sig = MOD && a.mod.pb != nullptr;
  m.keep = MOD ? a.mod.keep : 0;
#pragma unroll
  for (int g = 0; g < QG; ++g) m.pb[g] = m.sig ? a.mod.pb[head[g]] : 0.f;
  return m;
}

__device__ __forceinline__ bf16x8 ld16(const bf16_t* p) {
  const uint4 v = *reinterpret_cast<const uint4*>(p);
  return __builtin_bit_cast(bf16x8, v);
}
// For the pages that decoding reads once: a load that tells the caches so.  Measured on a plain read of 1 GiB
// whose instructions take whole lines of 128 bytes: 6.8 TB/s with this hint, 4.7 without.
__device__ __forceinline__ u32x4 ld16_once(const bf16_t* p) {
  return __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(p));
}
// Lanes l and l ^ 8 (the same quarter c = l / 16, rows r and r ^ 8 of a block of 16 rows) fetched whole lines: lane
// (r, c) chunk c + 4 (r / 8) of the block's row r % 8 into t0 and of row 8 + r % 8 into t1.  Afterwards t0 is chunk c
// and t1 chunk c + 4 of the lane's own row r: the operands of two consecutive 16x16x32 products.
__device__ __forceinline__ void to_own_row(u32x4& t0, u32x4& t1) {
  u32x4 s0, s1;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    // row_ror:8 reads lane l ^ 8 of each row of 16 lanes; the bank mask says which lanes take it (0xc: 8..15, 0x3: 0..7)
    s0[i] = __builtin_amdgcn_update_dpp(t0[i], t1[i], 0x128, 0xf, 0xc, false);
    s1[i] = __builtin_amdgcn_update_dpp(t1[i], t0[i], 0x128, 0xf, 0x3, false);
  }
  t0 = s0;
  t1 = s1;
}
__device__ __forceinline__ bf16x8 zero16() {
  const uint4 v = make_uint4(0, 0, 0, 0);
  return __builtin_bit_cast(bf16x8, v);
}
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
__device__ __forceinline__ uint32_t pack2(float a, float b) {      // round to nearest even, one instruction for the pair
  const bf16x2 v = {(__bf16)a, (__bf16)b};
  return __builtin_bit_cast(uint32_t, v);
}
__device__ __forceinline__ float group_max(float v) {     // over the four lanes that share l % 16
  v = fmaxf(v, __shfl_xor(v, 16, 64));
  return fmaxf(v, __shfl_xor(v, 32, 64));
}
__device__ __forceinline__ float group_sum(float v) {
  v += __shfl_xor(v, 16, 64);
  return v + __shfl_xor(v, 32, 64);
}


// Where the workgroup's tiles lie in LDS when the head size is 64, 128 or 256 (rows of 8, 16 or 32 chunks of 16
// bytes, no padding): chunk ch of key row `row` at chunk ch ^ g(row), where g numbers the 16 rows that one
// operand read touches (rows r % 4 + 8 (r / 4) + const) 0..15, or 0..7 twice for rows of 8 chunks; chunk ch of value
// row d (64 positions, 8 chunks) at chunk ch ^ (d & 7).  Measured: such reads run at about 210 bytes per clock
// and compute unit, rows padded by 16 bytes at about 120.
template <int DT>
__device__ __forceinline__ int k_swz(int row, int ch) {
  // (rows whose number of chunks is no power of two, a head of 192: the lowest three bits of ch only, which stays in the row)
  const int g = DT == 4 ? (((row >> 1) & 1) | (((row >> 3) & 3) << 1))
              : (2 * DT) & (2 * DT - 1) ? ((row & 3) | (((row >> 3) & 1) << 2)) : ((row & 3) | (((row >> 3) & 3) << 2));
  return row * (16 * DT) + ((ch ^ g) << 3);
}
__device__ __forceinline__ int v_swz(int d, int ch) { return d * TILE + ((ch ^ (d & 7)) << 3); }

// The part of a tile between its two products, for QG groups of 16 columns: s holds the tile's scores (rows of
// block jt as tile_step says); afterwards m_run, l_run and o are brought to the new running maximum and pf holds the
// probabilities 2^(s * scale2 - m) as the operand of the second product.
template <int DT, int QG, bool MOD>
__device__ __forceinline__ void softmax_tile(f32x4 (&s)[QG][4], f32x4 (&o)[QG][DT], float (&m_run)[QG], float (&l_run)[QG],
                                             int pos0, const int (&p_q)[QG], const int (&lo_q)[QG], float scale2,
                                             bool masked, bf16x8 (&pf)[2][QG], const ColMod<QG, MOD>& cm) {
  const int c = (threadIdx.x % 64) / 16;
  if constexpr (MOD) {
    // a cap or a distance bias: the scores are brought to their final value in natural units here, and only the
    // change of base is left to the factor below
#pragma unroll
    for (int g = 0; g < QG; ++g)
#pragma unroll
      for (int jt = 0; jt < 4; ++jt)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
          const int key = pos0 + 32 * (jt / 2) + 8 * c + 4 * (jt % 2) + v;
          s[g][jt][v] = mod_score_fast(s[g][jt][v] * cm.scale, cm.cap, cm.biased, cm.r1[g], cm.r2[g], p_q[g] - key);
        }
    scale2 = LOG2E;
  }
  // mask, running maximum, probabilities
#pragma unroll
  for (int g = 0; g < QG; ++g) {
    float m_tile = -INFINITY;
    if (masked) {
#pragma unroll
      for (int jt = 0; jt < 4; ++jt)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
          const int key = pos0 + 32 * (jt / 2) + 8 * c + 4 * (jt % 2) + v;
          const bool ok = MOD ? sees(key, p_q[g], lo_q[g], cm.keep) : (key <= p_q[g] && key >= lo_q[g]);
          s[g][jt][v] = ok ? s[g][jt][v] : -INFINITY;
          m_tile = fmaxf(m_tile, s[g][jt][v]);
        }
    } else {
#pragma unroll
      for (int jt = 0; jt < 4; ++jt)
#pragma unroll
        for (int v = 0; v < 4; ++v) m_tile = fmaxf(m_tile, s[g][jt][v]);
    }
    if constexpr (MOD) {
      if (cm.sig) {
        // sigmoid weights: 1 / (1 + e^-(s + pb)); a masked score of -inf gives 1 / inf = 0.  The running maximum stays at
        // 0, where it started, so nothing that came before is rescaled, and the sum is kept but never divided by.
        float l_sig = 0.f;
#pragma unroll
        for (int jt = 0; jt < 4; ++jt)
#pragma unroll
          for (int v = 0; v < 4; ++v) {
            const float p = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-LOG2E * (s[g][jt][v] + cm.pb[g])));
            s[g][jt][v] = p;
            l_sig += p;
          }
        l_run[g] += group_sum(l_sig);
        continue;
      }
    }
    m_tile = group_max(m_tile) * scale2;
    const float m_new = fmaxf(m_run[g], m_tile);
    const bool any = m_new != -INFINITY;
    const float alpha = any && m_run[g] != -INFINITY ? __builtin_amdgcn_exp2f(m_run[g] - m_new) : (any ? 0.f : 1.f);
    const float m_use = any ? m_new : 0.f;       // 2^(-inf - 0) = 0 for masked keys, also when all are masked
    float l_tile = 0.f;
#pragma unroll
    for (int jt = 0; jt < 4; ++jt)
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const float p = __builtin_amdgcn_exp2f(fmaf(s[g][jt][v], scale2, -m_use));
        s[g][jt][v] = p;
        l_tile += p;
      }
    l_run[g] = l_run[g] * alpha + group_sum(l_tile);
    m_run[g] = m_new;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int v = 0; v < 4; ++v) o[g][dt][v] *= alpha;
  }
  // the probabilities as the second product's operand: what the lane holds already
#pragma unroll
  for (int pr = 0; pr < 2; ++pr)
#pragma unroll
    for (int g = 0; g < QG; ++g) {
      const u32x4 pw = {pack2(s[g][2 * pr][0], s[g][2 * pr][1]), pack2(s[g][2 * pr][2], s[g][2 * pr][3]),
                        pack2(s[g][2 * pr + 1][0], s[g][2 * pr + 1][1]), pack2(s[g][2 * pr + 1][2], s[g][2 * pr + 1][3])};
      pf[pr][g] = __builtin_bit_cast(bf16x8, pw);
    }
}

// One tile of 64 positions for QG groups of 16 columns that share the tile's keys and values.  kt: the tile's
// keys, row i at kt + i * k_stride; vt: the tile's values transposed, dimension d at vt + d * v_stride (memory or
// LDS).  DT: number of 16-wide blocks of hd held in registers (hd <= 16 * DT).  p_q: position of this lane's
// column in each group (-1: no such column), lo_q: first position it may see; masked: whether any column of the
// wave has a key in this tile that it may not see (if not, the comparisons are left out).  qf: the columns'
// queries, 8 values of hd per 32-wide step at 8 * (l / 16).  Every operand read from kt and vt serves all QG
// groups.  EXACT: hd is exactly 16 DT and DT is even.  SWZ: kt and vt are tiles in LDS laid out by k_swz, v_swz.
// ONCE (with EXACT, tiles in memory that nothing else reads): keys and values are fetched by whole lines of 128
// bytes, eight lanes to a row, and lanes l and l ^ 8 exchange what belongs to the other's row.
// scale2 = scale * log2(e) > 0: maxima are kept in that unit and probabilities are 2^(s * scale2 - m), which is
// exp(s * scale - max) with one instruction for the power.
// VD, dt0: the wave sums the VD blocks of 16 value dimensions from block dt0 on (all DT of them unless a step's waves
// share a head's value dimensions among them); the scores are over all of hd either way.
// DIFF: groups of even number are columns of map 1, whose keys are the first half of a row, those of odd number of map 2.
template <int DT, int QG, bool EXACT, bool SWZ = false, bool ONCE = false, bool MOD = false, int VD = DT, bool DIFF = false>
__device__ __forceinline__ void tile_step(f32x4 (&o)[QG][VD], float (&m_run)[QG], float (&l_run)[QG],
                                          const bf16x8 (&qf)[QG][(DT + 1) / 2], const bf16_t* kt, int k_stride,
                                          const bf16_t* vt, int v_stride, int hd, int pos0, const int (&p_q)[QG],
                                          const int (&lo_q)[QG], float scale2, bool masked, const ColMod<QG, MOD>& cm,
                                          int dt0 = 0) {
  constexpr int KS = (DT + 1) / 2;
  const int lane = threadIdx.x % 64, r = lane % 16, c = lane / 16;
  // EXACT: hd == 16 DT with DT even, so nothing below depends on hd and every product is unconditional
  const int n_dt = EXACT ? DT : hd / 16, n_ks = EXACT ? KS : (hd + 31) / 32;
  static_assert(!ONCE || (EXACT && !SWZ), "whole lines need rows of whole lines, in memory");
  const int r8 = r % 8, q8 = (c + 4 * (r / 8)) * 8;      // ONCE: this lane fetches chunk q8 / 8 of rows r8 and 8 + r8
  f32x4 s[QG][4];
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
#pragma unroll
    for (int g = 0; g < QG; ++g) s[g][jt] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (ONCE) {
      const int row_a = 32 * (jt / 2) + 8 * (r8 / 4) + 4 * (jt % 2) + r8 % 4, row_b = row_a + 16;
      constexpr int KG = KS > 8 ? 8 : KS;      // steps of hd whose keys a lane holds at a time (heads beyond 256: half of them)
#pragma unroll
      for (int k0 = 0; k0 < KS; k0 += KG) {
        u32x4 kf[KG];
#pragma unroll
        for (int p = 0; p < KG / 2; ++p) {
          kf[2 * p] = ld16_once(kt + row_a * k_stride + 64 * (k0 / 2 + p) + q8);
          kf[2 * p + 1] = ld16_once(kt + row_b * k_stride + 64 * (k0 / 2 + p) + q8);
        }
#pragma unroll
        for (int p = 0; p < KG / 2; ++p) to_own_row(kf[2 * p], kf[2 * p + 1]);
#pragma unroll
        for (int ks = 0; ks < KG; ++ks)
#pragma unroll
          for (int g = 0; g < QG; ++g)
            s[g][jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, kf[ks]), qf[g][k0 + ks], s[g][jt], 0, 0, 0);
      }
      continue;
    }
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      if (ks < n_ks) {
        const int d0 = 32 * ks + 8 * c;
        const int krow = 32 * (jt / 2) + 8 * (r / 4) + 4 * (jt % 2) + r % 4;
        const bf16x8 kf = SWZ ? ld16(kt + k_swz<DT>(krow, 4 * ks + c))
                              : (EXACT || d0 < hd ? ld16(kt + krow * k_stride + d0) : zero16());
#pragma unroll
        for (int g = 0; g < QG; ++g)
          if (!(DIFF && EXACT) || (ks < KS / 2) == (g % 2 == 0))      // (where the halves do not fall between steps, queries have zeros)
            s[g][jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[g][ks], s[g][jt], 0, 0, 0);
      }
    }
  }
  bf16x8 pf[2][QG];
  softmax_tile<VD, QG, MOD>(s, o, m_run, l_run, pos0, p_q, lo_q, scale2, masked, pf, cm);
  if (ONCE) {
    // a row of values (64 positions of one dimension) is one line: both halves of the tile come with it
#pragma unroll
    for (int dt = 0; dt < VD; ++dt) {
      u32x4 v0 = ld16_once(vt + (16 * (dt0 + dt) + r8) * v_stride + q8), v1 = ld16_once(vt + (16 * (dt0 + dt) + 8 + r8) * v_stride + q8);
      to_own_row(v0, v1);
#pragma unroll
      for (int g = 0; g < QG; ++g) {
        o[g][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, v0), pf[0][g], o[g][dt], 0, 0, 0);
        o[g][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, v1), pf[1][g], o[g][dt], 0, 0, 0);
      }
    }
    return;
  }
#pragma unroll
  for (int pr = 0; pr < 2; ++pr) {
#pragma unroll
    for (int dt = 0; dt < VD; ++dt) {
      if (dt0 + dt < n_dt) {
        const bf16x8 vf = SWZ ? ld16(vt + v_swz(16 * (dt0 + dt) + r, 4 * pr + c))
                              : ld16(vt + (16 * (dt0 + dt) + r) * v_stride + 32 * pr + 8 * c);
#pragma unroll
        for (int g = 0; g < QG; ++g) o[g][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[pr][g], o[g][dt], 0, 0, 0);
      }
    }
  }
}

// Runs the wave's 16 columns over tiles [tile_beg, tile_end) straight from the cache pages.
template <int DT, bool EXACT, bool MOD, int VD = DT>
__device__ __forceinline__ void attend(f32x4 (&o)[1][VD], float (&m_run)[1], float (&l_run)[1],
                                       const bf16x8 (&qf)[1][(DT + 1) / 2], const bf16_t* kh, const bf16_t* vh,
                                       const int* table, int page_size, int64_t page_stride, int hd, int tile_beg,
                                       int tile_end, int p, bool valid, int lo_q, float scale2, const ColMod<1, MOD>& cm,
                                       int dt0 = 0) {
  const int pq[1] = {valid ? p : -1}, lq[1] = {lo_q};
  for (int tile = tile_beg; tile < tile_end; ++tile) {
    const int pos0 = tile * TILE;
    const int page = table[pos0 / page_size];
    const int in_page = pos0 % page_size;
    const bf16_t* kt = kh + (int64_t)page * page_stride + (int64_t)in_page * hd;      // [row][hd]
    const bf16_t* vt = vh + (int64_t)page * page_stride + in_page;                     // [hd][row]
    const bool masked = pos0 + TILE - 1 > p || pos0 < lo_q;      // the same for all lanes
    tile_step<DT, 1, EXACT, false, EXACT, MOD, VD>(o, m_run, l_run, qf, kt, hd, vt, page_size, hd, pos0, pq, lq, scale2, masked, cm, dt0);
  }
}

// The same run of tiles for a step that has few waves (a handful of sequences): then a wave has a SIMD's registers
// to itself, and keeps a whole tile of keys and values in them (2 DT registers of 16 bytes each, fetched by whole
// lines as in tile_step) while it works on the tile before.  Every product and sum is the one of `attend`, in the same
// order: only the loads go out earlier.
template <int DT>
struct TileRegs {
  u32x4 k[4][DT / 2];       // block jt, step ks of hd (before the exchange between lanes)
  u32x4 v[DT][2];           // block dt of hd, the two halves of the tile's positions
};
template <int DT>
__device__ __forceinline__ void fetch_tile(TileRegs<DT>& t, const bf16_t* kt, int k_stride, const bf16_t* vt, int v_stride) {
  const int lane = threadIdx.x % 64, r = lane % 16, c = lane / 16;
  const int r8 = r % 8, q8 = (c + 4 * (r / 8)) * 8;
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    const int row_a = 32 * (jt / 2) + 8 * (r8 / 4) + 4 * (jt % 2) + r8 % 4, row_b = row_a + 16;
#pragma unroll
    for (int p = 0; p < DT / 4; ++p) {
      t.k[jt][2 * p] = ld16_once(kt + row_a * k_stride + 64 * p + q8);
      t.k[jt][2 * p + 1] = ld16_once(kt + row_b * k_stride + 64 * p + q8);
    }
  }
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
    t.v[dt][0] = ld16_once(vt + (16 * dt + r8) * v_stride + q8);
    t.v[dt][1] = ld16_once(vt + (16 * dt + 8 + r8) * v_stride + q8);
  }
}
template <int DT, bool MOD>
__device__ __forceinline__ void tile_step_regs(f32x4 (&o)[1][DT], float (&m_run)[1], float (&l_run)[1],
                                               const bf16x8 (&qf)[1][DT / 2], TileRegs<DT>& t, int pos0,
                                               const int (&p_q)[1], const int (&lo_q)[1], float scale2, bool masked,
                                               const ColMod<1, MOD>& cm) {
  f32x4 s[1][4];
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    s[0][jt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int p = 0; p < DT / 4; ++p) to_own_row(t.k[jt][2 * p], t.k[jt][2 * p + 1]);
#pragma unroll
    for (int ks = 0; ks < DT / 2; ++ks)
      s[0][jt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, t.k[jt][ks]), qf[0][ks], s[0][jt], 0, 0, 0);
  }
  bf16x8 pf[2][1];
  softmax_tile<DT, 1, MOD>(s, o, m_run, l_run, pos0, p_q, lo_q, scale2, masked, pf, cm);
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
    to_own_row(t.v[dt][0], t.v[dt][1]);
    o[0][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, t.v[dt][0]), pf[0][0], o[0][dt], 0, 0, 0);
    o[0][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, t.v[dt][1]), pf[1][0], o[0][dt], 0, 0, 0);
  }
}
template <int DT, bool MOD>
__device__ __forceinline__ void attend_ahead(f32x4 (&o)[1][DT], float (&m_run)[1], float (&l_run)[1],
                                             const bf16x8 (&qf)[1][DT / 2], const bf16_t* kh, const bf16_t* vh,
                                             const int* table, int page_size, int64_t page_stride, int tile_beg,
                                             int tile_end, int p, bool valid, int lo_q, float scale2, const ColMod<1, MOD>& cm) {
  constexpr int hd = 16 * DT;
  const int pq[1] = {valid ? p : -1}, lq[1] = {lo_q};
  TileRegs<DT> t0, t1;
#define TQ_FETCH_TILE(regs, tile)                                                                          \
  do {                                                                                                     \
    const int pos0_ = (tile) * TILE;                                                                       \
    const int64_t base_ = (int64_t)table[pos0_ / page_size] * page_stride;                                 \
    const int in_page_ = pos0_ % page_size;                                                                \
    fetch_tile<DT>(regs, kh + base_ + (int64_t)in_page_ * hd, hd, vh + base_ + in_page_, page_size);       \
  } while (0)
#define TQ_STEP_TILE(regs, tile)                                                                           \
  do {                                                                                                     \
    const int pos0_ = (tile) * TILE;                                                                       \
    const bool masked_ = pos0_ + TILE - 1 > p || pos0_ < lo_q;                                             \
    tile_step_regs<DT, MOD>(o, m_run, l_run, qf, regs, pos0_, pq, lq, scale2, masked_, cm);                     \
  } while (0)
  TQ_FETCH_TILE(t0, tile_beg);
  for (int tile = tile_beg; tile < tile_end; tile += 2) {
    if (tile + 1 < tile_end) TQ_FETCH_TILE(t1, tile + 1);
    TQ_STEP_TILE(t0, tile);
    if (tile + 1 < tile_end) {
      if (tile + 2 < tile_end) TQ_FETCH_TILE(t0, tile + 2);
      TQ_STEP_TILE(t1, tile + 1);
    }
  }
#undef TQ_FETCH_TILE
#undef TQ_STEP_TILE
}

template <int DT>
__device__ __forceinline__ void load_query(bf16x8 (&qf)[(DT + 1) / 2], const bf16_t* qrow, int hd, bool valid, int from = 0) {
  const int c = (threadIdx.x % 64) / 16;
#pragma unroll
  for (int ks = 0; ks < (DT + 1) / 2; ++ks) {
    const int d0 = 32 * ks + 8 * c;
    qf[ks] = valid && d0 >= from && d0 < hd ? ld16(qrow + d0) : zero16();      // (zeros in front of `from` and behind hd)
  }
}

// ------------------------------------------------------------------------------------------ whole prompts
// grid (blocks of 64 QG new tokens x heads x sequences), block 256: wave w takes tokens 16 QG w .. of its block,
// QG groups of 16.  The cache already holds the step's keys and values.  Blocks are numbered from the end of the
// sequences: a block attends to everything before it, so the longest ones start first and the short ones fill
// the gaps that they leave.  The workgroup brings each tile of keys and values into one of two LDS buffers
// (swizzled for head sizes 64, 128, 256; else key rows padded by KPAD and value rows VSTR long) while it works on
// the other, and the tile after that is on its way from memory into registers meanwhile: one barrier per tile.
#define KPAD 8
#define VSTR 72
#ifndef ATTN_TWO_BUFFERS_UP_TO
#define ATTN_TWO_BUFFERS_UP_TO 8      // heads of up to 16 times this many numbers keep two tiles in LDS
#endif

// Heads wider than 256 (DT = 32; an attention over compressed rows that all heads share has such): one buffer instead of
// two, since two tiles of 64 x 512 keys and values are beyond the LDS, and a wave to a SIMD, since a column's sums
// alone are 128 registers; the next tile still travels from memory into registers while this one is worked on.
// VD < DT: the values' first 16 VD dimensions alone are summed and written (zeros behind them up to hd): an attention
// whose keys are wider than its values, laid out at the keys' width.
// DIFF: two maps a head, a token's two columns in two groups of one lane; they are made one where the output is normalised.
template <int DT, int QG, bool EXACT, bool MOD, int VD = DT, bool DIFF = false>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DT > (DIFF ? 8 : 16) ? 1 : 2))) void attn_prefill_kernel(AttnArgs a, int n_blocks, int B, DiffArgs df) {
  constexpr bool ONEBUF = DT > ATTN_TWO_BUFFERS_UP_TO;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem_raw[];
  static_assert(!DIFF || (QG % 2 == 0 && !MOD && VD == DT), "two maps a head: in pairs of groups, with plain scores");
  constexpr int QW = 16 * (DIFF ? QG / 2 : QG);
  constexpr int KCH = (TILE * 2 * DT + 255) / 256;      // 16-byte chunks of a key tile per thread
  constexpr int VCH = (16 * VD * 8 + 255) / 256;        // and of a value tile
  static_assert(VD <= DT && (VD == DT || EXACT), "fewer value dimensions than key dimensions: for exact head sizes");
  const int hd = EXACT ? 16 * DT : a.hd, kcpr = hd / 8;
  // elements of one buffer: keys [TILE][hd + KPAD], values [hd][VSTR]; swizzled instead of padded when EXACT
  const int kstr = EXACT ? hd : hd + KPAD, vstr = EXACT ? TILE : VSTR;
  const int buf = TILE * kstr + (VD < DT ? 16 * VD : hd) * vstr;
  bf16_t* Ks = (bf16_t*)smem_raw;
  bf16_t* Vs = Ks + TILE * kstr;
  const int per_block = a.nh * B;
  const int blk = n_blocks - 1 - (int)blockIdx.x / per_block;
  const int h = (int)blockIdx.x % per_block % a.nh, seq = (int)blockIdx.x % per_block / a.nh;
  const int tid = threadIdx.x, lane = tid % 64, wave = tid / 64, r = lane % 16, c = lane / 16;
  const int t0 = a.cu_seqlens[seq], n = a.cu_seqlens[seq + 1] - t0;
  const int qb = blk * 4 * QW;
  if (qb >= n) return;
  const int start = a.start[seq];
  const int kvh = h / (a.nh / a.nkv);
  const int64_t head_off = (int64_t)kvh * a.page_size * hd;
  const int* table = a.block_table + (size_t)a.slots[seq] * a.bt_stride;

  int p_q[QG], lo_q[QG];
  bf16x8 qf[QG][(DT + 1) / 2];
  f32x4 o[QG][VD];
  float m_run[QG], l_run[QG];
#pragma unroll
  for (int g = 0; g < QG; ++g) {
    const int qi = qb + wave * QW + (DIFF ? g / 2 : g) * 16 + r;
    const bool valid = qi < n;
    p_q[g] = valid ? start + qi : -1;
    lo_q[g] = reach_lo(p_q[g], a.window, a.mod.chunk);
    load_query<DT>(qf[g], a.q + ((size_t)(t0 + (valid ? qi : 0)) * a.nh + h) * hd, DIFF && g % 2 == 0 ? hd / 2 : hd, valid,
                   DIFF && g % 2 ? hd / 2 : 0);
#pragma unroll
    for (int dt = 0; dt < VD; ++dt) o[g][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
    m_run[g] = -INFINITY;
    l_run[g] = 0.f;
    if (a.mod.sink) {       // a score without key or value, counted once; maxima are in units of log2
      m_run[g] = a.mod.sink[h] * LOG2E;
      l_run[g] = 1.f;
    }
    if (MOD && a.mod.pb) m_run[g] = 0.f;
  }
  // tiles the workgroup goes through, and those among them that this wave's tokens can see
  const int wg_first = start + qb, wg_last = start + min(qb + 4 * QW, n) - 1;
  // (kept first positions: their tiles come first, then the walk jumps to the first tile of the workgroup's windows)
  const int kept = MOD ? keep_tiles(a.mod.keep, TILE) : 0;
  const int lo_tile = reach_lo(wg_first, a.window, a.mod.chunk) / TILE;
  const int tile_beg = first_tile(lo_tile, kept), tile_end = wg_last / TILE + 1;
  auto after = [&](int t) { return next_tile(t, lo_tile, kept); };
  const int wq0 = qb + wave * QW;
  const bool wave_has = wq0 < n;
  const int wave_first = start + wq0, wave_last = start + min(wq0 + QW, n) - 1;
  const int wave_lo_last = reach_lo(wave_last, a.window, a.mod.chunk);     // first key of the wave's last token
  const int wave_beg = reach_lo(wave_first, a.window, a.mod.chunk) / TILE;
  int heads_g[QG];
#pragma unroll
  for (int g = 0; g < QG; ++g) heads_g[g] = h;
  const ColMod<QG, MOD> cm = col_mod<QG, MOD>(a, heads_g);
  const int wave_end = wave_has ? wave_last / TILE + 1 : 0;

  // what this thread carries of every tile: where its chunks lie in the tile in memory and in LDS (a thread
  // past the end of a small tile carries the last chunk once more)
  // (with one buffer the places are worked out anew at every use: 4 (KCH + VCH) registers are more than a wave can spare there)
  constexpr int NIDX = ONEBUF ? 1 : (KCH > VCH ? KCH : VCH);
  int k_g_[NIDX], k_l_[NIDX], v_g_[NIDX], v_l_[NIDX];
  auto k_place = [&](int j, int& in_mem, int& in_lds) {
    const int i = min(tid + j * 256, TILE * kcpr - 1), row = i / kcpr, ch = i % kcpr;
    in_mem = row * hd + ch * 8;
    in_lds = EXACT ? k_swz<DT>(row, ch) : row * kstr + ch * 8;
  };
  auto v_place = [&](int j, int& in_mem, int& in_lds) {
    const int i = min(tid + j * 256, (VD < DT ? 16 * VD : hd) * 8 - 1), d = i / 8, ch = i % 8;
    in_mem = d * a.page_size + ch * 8;
    in_lds = EXACT ? v_swz(d, ch) : d * vstr + ch * 8;
  };
  if constexpr (!ONEBUF) {
#pragma unroll
    for (int j = 0; j < KCH; ++j) k_place(j, k_g_[j], k_l_[j]);
#pragma unroll
    for (int j = 0; j < VCH; ++j) v_place(j, v_g_[j], v_l_[j]);
  }
  auto k_g = [&](int j) { if constexpr (ONEBUF) { int m, l; k_place(j, m, l); return m; } else return k_g_[j]; };
  auto k_l = [&](int j) { if constexpr (ONEBUF) { int m, l; k_place(j, m, l); return l; } else return k_l_[j]; };
  auto v_g = [&](int j) { if constexpr (ONEBUF) { int m, l; v_place(j, m, l); return m; } else return v_g_[j]; };
  auto v_l = [&](int j) { if constexpr (ONEBUF) { int m, l; v_place(j, m, l); return l; } else return v_l_[j]; };
  u32x4 pk[KCH], pv[VCH];
  const int tiles_per_page = a.page_size / TILE;
  int page_next = table[tile_beg / tiles_per_page];     // page of the tile that the next fetch takes
#define TQ_FETCH(tile, nxt)                                                                                 \
  do {                                                                                                      \
    const int64_t base = head_off + (int64_t)page_next * a.page_stride;                                     \
    const int in_page = ((tile) % tiles_per_page) * TILE;                                                   \
    const bf16_t* kg = a.k_pool + base + (int64_t)in_page * hd;                                             \
    const bf16_t* vg = a.v_pool + base + in_page;                                                           \
    _Pragma("unroll") for (int j = 0; j < KCH; ++j) pk[j] = *reinterpret_cast<const u32x4*>(kg + k_g(j));   \
    _Pragma("unroll") for (int j = 0; j < VCH; ++j) pv[j] = *reinterpret_cast<const u32x4*>(vg + v_g(j));   \
    if ((nxt) < tile_end) page_next = table[(nxt) / tiles_per_page];                                        \
  } while (0)
#define TQ_STAGE(off)                                                                                       \
  do {                                                                                                      \
    _Pragma("unroll") for (int j = 0; j < KCH; ++j) *reinterpret_cast<u32x4*>(Ks + (off) + k_l(j)) = pk[j]; \
    _Pragma("unroll") for (int j = 0; j < VCH; ++j) *reinterpret_cast<u32x4*>(Vs + (off) + v_l(j)) = pv[j]; \
  } while (0)

  TQ_FETCH(tile_beg, after(tile_beg));
  if constexpr (ONEBUF) {
    for (int tile = tile_beg; tile < tile_end; tile = after(tile)) {
      const int t1 = after(tile);
      TQ_STAGE(0);
      if (t1 < tile_end) TQ_FETCH(t1, after(t1));
      __syncthreads();
      if ((tile >= wave_beg || tile < kept) && tile < wave_end) {
        const int pos0 = tile * TILE;
        const bool masked = pos0 + TILE - 1 > wave_first || pos0 < wave_lo_last;
        tile_step<DT, QG, EXACT, EXACT, false, MOD, VD, DIFF>(o, m_run, l_run, qf, Ks, kstr, Vs, vstr, hd, pos0, p_q, lo_q,
                                        a.scale * LOG2E, masked, cm);
      }
      __syncthreads();
    }
  } else {
  TQ_STAGE(0);
  if (after(tile_beg) < tile_end) TQ_FETCH(after(tile_beg), after(after(tile_beg)));
  __syncthreads();
  int cur = 0;
  for (int tile = tile_beg; tile < tile_end; tile = after(tile), cur ^= buf) {
    const int t1 = after(tile), t2 = after(t1);
    if (t1 < tile_end) {
      TQ_STAGE(cur ^ buf);
      if (t2 < tile_end) TQ_FETCH(t2, after(t2));
    }
    if ((tile >= wave_beg || tile < kept) && tile < wave_end) {
      const int pos0 = tile * TILE;
      const bool masked = pos0 + TILE - 1 > wave_first || pos0 < wave_lo_last;
      tile_step<DT, QG, EXACT, EXACT, false, MOD, VD, DIFF>(o, m_run, l_run, qf, Ks + cur, kstr, Vs + cur, vstr, hd, pos0, p_q, lo_q,
                                      a.scale * LOG2E, masked, cm);
    }
    __syncthreads();
  }
  }
#undef TQ_FETCH
#undef TQ_STAGE
  if constexpr (DIFF) {
#pragma unroll
    for (int g = 0; g < QG; g += 2) {
      const float i1 = 1.0f / l_run[g], i2 = -df.lambda / l_run[g + 1];
      float ss = 0.f;
#pragma unroll
      for (int dt = 0; dt < DT; ++dt)
        if (16 * dt < hd)
#pragma unroll
          for (int v = 0; v < 4; ++v) {
            const float x = fmaf(o[g][dt][v], i1, o[g + 1][dt][v] * i2);
            o[g][dt][v] = x;
            ss = fmaf(x, x, ss);
          }
      ss = group_sum(ss);      // (before lanes without a token leave: the four lanes of a column have it or not together)
      if (p_q[g] < 0) continue;
      const float f = df.post / sqrtf(ss / (float)df.vd + df.eps);
      const size_t t = t0 + p_q[g] - start;
      bf16_t* orow = a.out + t * a.ldo + (size_t)h * hd;
      const float* gr = df.gate ? df.gate + t * df.ld_gate + (size_t)h * hd : nullptr;
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        if (16 * dt < hd) {
          f32x4 x = o[g][dt] * f;
          if (gr) {
            const f32x4 z = *reinterpret_cast<const f32x4*>(gr + 16 * dt + 4 * c);
#pragma unroll
            for (int v = 0; v < 4; ++v) x[v] /= 1.0f + expf(-z[v]);
          }
          *reinterpret_cast<u32x2*>(orow + 16 * dt + 4 * c) = u32x2{pack2(x[0], x[1]), pack2(x[2], x[3])};
        }
      }
    }
    return;
  }
#pragma unroll
  for (int g = 0; g < QG; ++g) {
    if (p_q[g] < 0) continue;
    float inv = (MOD && a.mod.pb) ? 1.0f : 1.0f / l_run[g];
    if (a.head_gate) inv /= 1.0f + expf(-a.head_gate[(size_t)(t0 + p_q[g] - start) * a.ld_gate + h]);
    bf16_t* orow = a.out + (size_t)(t0 + p_q[g] - start) * a.ldo + (size_t)h * hd;
#pragma unroll
    for (int dt = 0; dt < VD; ++dt) {
      if (16 * dt < hd) {
        const u32x2 w = {pack2(o[g][dt][0] * inv, o[g][dt][1] * inv), pack2(o[g][dt][2] * inv, o[g][dt][3] * inv)};
        *reinterpret_cast<u32x2*>(orow + 16 * dt + 4 * c) = w;
      }
    }
#pragma unroll
    for (int dt = VD; dt < DT; ++dt) *reinterpret_cast<u32x2*>(orow + 16 * dt + 4 * c) = u32x2{0u, 0u};
  }
}

// ------------------------------------------------------------------------------------------ decoding
// One new token per sequence at position start[b].  grid (runs, nkv * ceil(g / 16), B), block 64: the wave
// takes run x (tiles S x .. S x + S - 1, S = tiles_per_run(position)) for up to 16 of the g = nh / nkv heads of one kv head and
// writes their unnormalised sums with maximum and denominator.  The grid has the runs of the step's longest
// sequence, so that no wave is started for nothing where all sequences are about as long (a wave that finds no run
// costs as much to start as one that does: a third more of them made the kernel a fifth slower).  A shorter
// sequence of the same step may still have more runs than that, positions below 4096 being cut finer: its waves
// then take the further runs in turn (wave x the runs x, x + the grid's runs, ...), each into its own place, so
// that no wave has more than one or two of them (left to the last wave alone, 30 runs in a row made a step with
// one sequence beyond position 4096 and seven shorter ones a third slower).
// AHEAD (with EXACT): the form for steps of few waves, which fetches a tile ahead (attend_ahead).
// VS: the waves of a run that share a head's value dimensions among them (heads beyond 256: four, each with the scores of
// the whole head and a quarter of the sums, so that a step has four times the waves and none holds 128 registers of sums).
template <int DT, bool EXACT, bool AHEAD = false, bool MOD = false, int VS = 1>
__global__ __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(AHEAD ? 1 : (DT > 8 ? 2 : 3)))) void attn_decode_kernel(AttnArgs a) {
  static_assert(DT % VS == 0 && (VS == 1 || !AHEAD), "the value dimensions are shared in whole blocks");
  constexpr int VD = DT / VS;
  const int b = blockIdx.z;
  const int g = a.nh / a.nkv, ngc = (g + 15) / 16;
  const int dt0 = (int)(blockIdx.y % VS) * VD, y = blockIdx.y / VS;
  const int kvh = y / ngc, cg = y % ngc;
  const int lane = threadIdx.x, r = lane % 16, c = lane / 16;
  const int p = a.start[b];
  const int lo = reach_lo(p, a.window, a.mod.chunk);
  const int S = tiles_per_run(p), n_runs = runs_at(p);
  if ((int)blockIdx.x >= n_runs) return;
  const int hg = cg * 16 + r;                 // head within the group
  const bool valid = hg < g;
  const int h = kvh * g + (valid ? hg : 0);
  const int64_t head_off = (int64_t)kvh * a.page_size * a.hd;
  const int* table = a.block_table + (size_t)a.slots[b] * a.bt_stride;
  const int t = a.cu_seqlens[b];
  const int head1[1] = {h};
  const ColMod<1, MOD> cm = col_mod<1, MOD>(a, head1);

  bf16x8 qf[1][(DT + 1) / 2];
  load_query<DT>(qf[0], a.q + ((size_t)t * a.nh + h) * a.hd, a.hd, valid);
  // tiles of kept first positions that lie before the window's first tile: a run takes its share of them before its
  // share of the window's tiles
  const int kept_before = MOD ? min(keep_tiles(a.mod.keep, TILE), lo / TILE) : 0;
  for (int run = blockIdx.x; run < n_runs; run += gridDim.x) {
    const int tile_beg = max(run * S, lo / TILE), tile_end = min((run + 1) * S, p / TILE + 1);
    const int kept_beg = run * S, kept_end = min(tile_end, kept_before);
    if (tile_beg >= tile_end && kept_beg >= kept_end) continue;       // all of the run lies before the window
    f32x4 o[1][VD];
#pragma unroll
    for (int dt = 0; dt < VD; ++dt) o[0][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m_run[1] = {(MOD && a.mod.pb) ? 0.f : -INFINITY}, l_run[1] = {0.f};
#pragma unroll
    for (int part = MOD ? 0 : 1; part < 2; ++part) {
      const int beg = part ? tile_beg : kept_beg, end = part ? tile_end : kept_end;
      if (beg >= end) continue;
      if constexpr (AHEAD)
        attend_ahead<DT, MOD>(o, m_run, l_run, qf, a.k_pool + head_off, a.v_pool + head_off, table, a.page_size, a.page_stride,
                         beg, end, p, valid, lo, a.scale * LOG2E, cm);
      else
        attend<DT, EXACT, MOD, VD>(o, m_run, l_run, qf, a.k_pool + head_off, a.v_pool + head_off, table, a.page_size, a.page_stride,
                          a.hd, beg, end, p, valid, lo, a.scale * LOG2E, cm, dt0);
    }
    if (!valid) continue;
    float* out = a.partial + (((size_t)b * a.nh + h) * a.max_runs + run) * (a.hd + 2);
#pragma unroll
    for (int dt = 0; dt < VD; ++dt) {
      if (16 * (dt0 + dt) < a.hd) {
#pragma unroll
        for (int v = 0; v < 4; ++v) out[16 * (dt0 + dt) + 4 * c + v] = o[0][dt][v];
      }
    }
    if (c == 0 && dt0 == 0) {
      out[a.hd] = m_run[0];
      out[a.hd + 1] = l_run[0];
    }
  }
}

// Joins the runs of one (sequence, head) in order of position: grid (nh, B), block 64.  The weights
// 2^(m_s - m) of the runs are worked out once, a lane per run, and kept in LDS; then every lane sums its
// dimensions over the runs in order.
#define MAX_RUNS_LDS 2048
// (heads of 128, 256, 384 or 512: a wave to every 128 dimensions, each working out the weights for itself, so that no
// wave waits for another)
__global__ __launch_bounds__(256) void attn_join_kernel(AttnArgs a) {
  extern __shared__ float wgt_all[];        // [waves][MAX_RUNS_LDS]
  const int h = blockIdx.x, b = blockIdx.y, lane = threadIdx.x % 64, wave = threadIdx.x / 64;
  float* wgt = wgt_all + wave * MAX_RUNS_LDS;
  const int p = a.start[b];
  const int lo = reach_lo(p, a.window, a.mod.chunk);
  const int S = tiles_per_run(p);
  int run_beg = lo / TILE / S;
  const int run_end = p / TILE / S + 1;
  // runs that hold kept first positions before the window's first tile come first, then the window's runs: entry i of
  // the walk is run RUN_OF(i)
  int kept_runs = (min(keep_tiles(a.mod.keep, TILE), lo / TILE) + S - 1) / S;
  if (kept_runs >= run_beg) run_beg = kept_runs = 0;
  const int n_runs = kept_runs + run_end - run_beg;
#define RUN_OF(i) ((i) < kept_runs ? (i) : run_beg + (i) - kept_runs)
  const int stride = a.hd + 2;
  const float* part = a.partial + ((size_t)b * a.nh + h) * a.max_runs * stride;
  float m = -INFINITY;
  for (int i = lane; i < n_runs; i += 64) m = fmaxf(m, part[(size_t)RUN_OF(i) * stride + a.hd]);
  m = wave_max(m);
  float l = 0.f;
  if (a.mod.sink) {         // the sink joins here, once, like one more run with a sum of 1 and no values
    m = fmaxf(m, a.mod.sink[h] * LOG2E);
    l = __builtin_amdgcn_exp2f(a.mod.sink[h] * LOG2E - m);
  }
  for (int i0 = 0; i0 < n_runs; i0 += 64) {     // denominators in run order, 64 runs at a time
    const int i = i0 + lane;
    float w = 0.f, wl = 0.f;
    if (i < n_runs) {
      const size_t s = RUN_OF(i);
      w = __builtin_amdgcn_exp2f(part[s * stride + a.hd] - m);      // maxima are in units of log2
      wl = w * part[s * stride + a.hd + 1];
      wgt[i] = w;
    }
    l += wave_sum(wl);
  }
  __builtin_amdgcn_wave_barrier();
  float inv = a.mod.pb ? 1.0f : 1.0f / l;       // sigmoid weights are not normalised (every run's maximum is 0)
  if (a.head_gate) inv /= 1.0f + expf(-a.head_gate[(size_t)a.cu_seqlens[b] * a.ld_gate + h]);
  bf16_t* orow = a.out + (size_t)a.cu_seqlens[b] * a.ldo + (size_t)h * a.hd;
  if (a.hd % 128 == 0) {      // a lane takes two neighbouring dimensions of its wave's 128: one pass over the runs, 8 bytes at a time
    const int d = 128 * wave + 2 * lane;
    float acc0 = 0.f, acc1 = 0.f;
#pragma unroll 8
    for (int i = 0; i < n_runs; ++i) {
      const float2 v = *reinterpret_cast<const float2*>(part + (size_t)RUN_OF(i) * stride + d);
      acc0 = fmaf(wgt[i], v.x, acc0);
      acc1 = fmaf(wgt[i], v.y, acc1);
    }
    *reinterpret_cast<uint32_t*>(orow + d) = pack2(acc0 * inv, acc1 * inv);
    return;
  }
  for (int d = lane; d < a.hd; d += 64) {
    float acc = 0.f;
#pragma unroll 8
    for (int i = 0; i < n_runs; ++i) acc = fmaf(wgt[i], part[(size_t)RUN_OF(i) * stride + d], acc);
    orow[d] = f32_to_bf16(acc * inv);
  }
#undef RUN_OF
}

// The same for two maps a head: a.nh counts the maps' columns (head h's maps are 2 h and 2 h + 1), grid (nh / 2, B), block 128:
// a wave joins a map's runs, then the first makes the two one.  A lane takes NP pairs of neighbouring dimensions (heads of up
// to 128 NP; every load is unconditional, from an address clamped into the row).
template <int NP>
__global__ __launch_bounds__(128) void attn_join_diff_kernel(AttnArgs a, DiffArgs df) {
  extern __shared__ float wgt_all[];        // [2][MAX_RUNS_LDS]
  __shared__ float other[128 * NP];
  const int h = blockIdx.x, b = blockIdx.y, lane = threadIdx.x % 64, map = threadIdx.x / 64;
  float* wgt = wgt_all + map * MAX_RUNS_LDS;
  const int n_runs = a.start[b] / TILE / tiles_per_run(a.start[b]) + 1, stride = a.hd + 2;
  const float* part = a.partial + ((size_t)b * a.nh + 2 * h + map) * a.max_runs * stride;
  float m = -INFINITY;
  for (int i = lane; i < n_runs; i += 64) m = fmaxf(m, part[(size_t)i * stride + a.hd]);
  m = wave_max(m);
  float l = 0.f;
  for (int i0 = 0; i0 < n_runs; i0 += 64) {
    const int i = i0 + lane;
    float w = 0.f, wl = 0.f;
    if (i < n_runs) {
      w = __builtin_amdgcn_exp2f(part[(size_t)i * stride + a.hd] - m);
      wl = w * part[(size_t)i * stride + a.hd + 1];
      wgt[i] = w;
    }
    l += wave_sum(wl);
  }
  __builtin_amdgcn_wave_barrier();
  const float inv = 1.0f / l;
  float2 acc[NP];
  int at[NP];
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    acc[j] = float2{0.f, 0.f};
    at[j] = min(128 * j + 2 * lane, a.hd - 2);
  }
#pragma unroll 8
  for (int i = 0; i < n_runs; ++i) {
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      const float2 v = *reinterpret_cast<const float2*>(part + (size_t)i * stride + at[j]);
      acc[j].x = fmaf(wgt[i], v.x, acc[j].x);
      acc[j].y = fmaf(wgt[i], v.y, acc[j].y);
    }
  }
  if (map == 1)
#pragma unroll
    for (int j = 0; j < NP; ++j) {
      other[128 * j + 2 * lane] = acc[j].x * inv;
      other[128 * j + 2 * lane + 1] = acc[j].y * inv;
    }
  __syncthreads();
  if (map == 1) return;
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const bool has = 128 * j + 2 * lane < a.hd;
    acc[j].x = has ? fmaf(acc[j].x, inv, -df.lambda * other[128 * j + 2 * lane]) : 0.f;
    acc[j].y = has ? fmaf(acc[j].y, inv, -df.lambda * other[128 * j + 2 * lane + 1]) : 0.f;
    ss = fmaf(acc[j].x, acc[j].x, fmaf(acc[j].y, acc[j].y, ss));
  }
  const float f = df.post / sqrtf(wave_sum(ss) / (float)df.vd + df.eps);
  const size_t t = a.cu_seqlens[b];
  bf16_t* orow = a.out + t * a.ldo + (size_t)h * a.hd;
  const float* gr = df.gate ? df.gate + t * df.ld_gate + (size_t)h * a.hd : nullptr;
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    if (128 * j + 2 * lane < a.hd) {
      const float2 z = gr ? *reinterpret_cast<const float2*>(gr + at[j]) : float2{0.f, 0.f};
      const float gx = gr ? 1.0f / (1.0f + expf(-z.x)) : 1.0f, gy = gr ? 1.0f / (1.0f + expf(-z.y)) : 1.0f;
      *reinterpret_cast<uint32_t*>(orow + at[j]) = pack2(acc[j].x * f * gx, acc[j].y * f * gy);
    }
  }
}

// ------------------------------------------------------------------------------------------ launch
template <int DT, int QG, bool EXACT, bool MOD, int VD = DT>
static int launch_prefill_as(const AttnArgs& a, int B, int max_new, hipStream_t st) {
  const size_t shmem = (DT > ATTN_TWO_BUFFERS_UP_TO ? 1 : 2) * (EXACT ? (size_t)TILE * (a.hd + 16 * VD) : (size_t)TILE * (a.hd + KPAD) + (size_t)a.hd * VSTR) * sizeof(bf16_t);
  if (shmem > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)attn_prefill_kernel<DT, QG, EXACT, MOD, VD>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem);
  const int n_blocks = (max_new + 64 * QG - 1) / (64 * QG);
  if ((int64_t)n_blocks * a.nh * B > 0x7fffffff) return TQ_ERR_UNSUPPORTED;
  hipLaunchKernelGGL((attn_prefill_kernel<DT, QG, EXACT, MOD, VD>), dim3(n_blocks * a.nh * B), dim3(256), shmem, st, a, n_blocks, B, DiffArgs{});
  return 0;
}
// (the kernels that cap or bias scores are instantiations of their own, so that the others carry nothing of it)
template <int DT, int QG, bool EXACT, int VD = DT>
static int launch_prefill(const AttnArgs& a, int B, int max_new, hipStream_t st) {
  return (a.mod.cap > 0.f || a.mod.r1 || a.mod.pb || a.mod.keep > 0) ? launch_prefill_as<DT, QG, EXACT, true, VD>(a, B, max_new, st)
                                       : launch_prefill_as<DT, QG, EXACT, false, VD>(a, B, max_new, st);
}
template <int DT, bool EXACT, bool MOD>
static void launch_decode_as(const AttnArgs& a, int B, int grid_runs, hipStream_t st, const DiffArgs* df = nullptr) {
  const int g = a.nh / a.nkv;
  const dim3 join_block(a.hd % 128 == 0 ? 64 * (a.hd / 128) : 64);      // a wave to every 128 dimensions of a head
  if constexpr (DT > 16) {
    hipLaunchKernelGGL((attn_decode_kernel<DT, EXACT, false, MOD, 4>), dim3(grid_runs, a.nkv * ((g + 15) / 16) * 4, B), dim3(64), 0, st, a);
  } else {
    const dim3 grid(grid_runs, a.nkv * ((g + 15) / 16), B);
    // at most a wave to a SIMD: each has the registers to fetch a tile ahead (one sequence at position 8,191: 2.38 ms a
    // step against 2.61; with more waves than that the form is no faster, from twice as many on slower)
    if (EXACT && DT <= 8 && (int64_t)grid.x * grid.y * grid.z <= 1024)
      hipLaunchKernelGGL((attn_decode_kernel<DT, EXACT, EXACT && DT <= 8, MOD>), grid, dim3(64), 0, st, a);
    else
      hipLaunchKernelGGL((attn_decode_kernel<DT, EXACT, false, MOD>), grid, dim3(64), 0, st, a);
  }
  if (df && a.hd <= 128)
    hipLaunchKernelGGL(attn_join_diff_kernel<1>, dim3(a.nh / 2, B), dim3(128), 2 * MAX_RUNS_LDS * sizeof(float), st, a, *df);
  else if (df)
    hipLaunchKernelGGL(attn_join_diff_kernel<2>, dim3(a.nh / 2, B), dim3(128), 2 * MAX_RUNS_LDS * sizeof(float), st, a, *df);
  else
    hipLaunchKernelGGL(attn_join_kernel, dim3(a.nh, B), join_block, join_block.x / 64 * MAX_RUNS_LDS * sizeof(float), st, a);
}
template <int DT, bool EXACT>
static void launch_decode(const AttnArgs& a, int B, int grid_runs, hipStream_t st) {
  if (a.mod.cap > 0.f || a.mod.r1 || a.mod.pb || a.mod.keep > 0) launch_decode_as<DT, EXACT, true>(a, B, grid_runs, st);
  else launch_decode_as<DT, EXACT, false>(a, B, grid_runs, st);
}

// Two maps a head.  Prompts: 16 tokens with both their maps to a wave.
template <int DT, bool EXACT>
static int launch_diff_prefill(const AttnArgs& a, const DiffArgs& df, int B, int max_new, hipStream_t st) {
  const size_t shmem = (DT > ATTN_TWO_BUFFERS_UP_TO ? 1 : 2) * (EXACT ? (size_t)TILE * (a.hd + 16 * DT) : (size_t)TILE * (a.hd + KPAD) + (size_t)a.hd * VSTR) * sizeof(bf16_t);
  if (shmem > 48 * 1024)
    (void)hipFuncSetAttribute((const void*)attn_prefill_kernel<DT, 2, EXACT, false, DT, true>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem);
  const int n_blocks = (max_new + 63) / 64;
  if ((int64_t)n_blocks * a.nh * B > 0x7fffffff) return TQ_ERR_UNSUPPORTED;
  hipLaunchKernelGGL((attn_prefill_kernel<DT, 2, EXACT, false, DT, true>), dim3(n_blocks * a.nh * B), dim3(256), shmem, st, a, n_blocks, B, df);
  return 0;
}

// Number of floats of `partial` that decoding B sequences up to position max_end needs.
TQ_API int64_t tq_attention_decode_scratch(int B, int nh, int hd, int max_end) {
  return (int64_t)B * nh * most_runs(max_end) * (hd + 2);
}

// decode != 0: every sequence brings exactly one token.  max_new: longest run of new tokens of a sequence;
// max_end: largest position + 1 that any token of the step has.
// softcap, r1, r2, chunk, sink: see score_mod.h (0, null, null, 0, null: nothing).
// value_width (0: hd): the values' first numbers that matter; a head's value rows behind them are zeros, and so is the
// output there, which lets a kernel leave them out.  head_gate (null: none), float [T][ld_gate]: the output of head h of
// token t is multiplied by sigmoid(head_gate[t][h]) where it is normalised, before it is rounded.
// pb, keep: sigmoid weights with a bias per head, and first positions that stay visible (score_mod.h; null, 0: neither).
// ldo: numbers between the rows of two tokens in out, a multiple of 4 (0: nh * hd).
TQ_API int tq_attention_mfma_ld(const void* q, const void* k_pool, const void* v_pool, const int* block_table,
                                       int bt_stride, const int* cu_seqlens, const int* slots, const int* start, int page_size,
                                       int64_t page_stride, int B, int nh, int nkv, int hd, int window, float scale,
                                       float softcap, const float* r1, const float* r2, int chunk, const float* sink,
                                       void* out, float* partial, int decode, int max_new, int max_end, int value_width,
                                       const float* head_gate, int64_t ld_gate, const float* pb, int keep, int64_t ldo,
                                       hipStream_t st) {
  if (B <= 0) return 0;
  if (ldo == 0) ldo = (int64_t)nh * hd;
  if (ldo < (int64_t)nh * hd || ldo % 4 != 0) return TQ_ERR_BAD_ARG;
  if ((r1 == nullptr) != (r2 == nullptr) || chunk < 0 || softcap < 0.f || value_width < 0 || value_width > hd || (head_gate && ld_gate < nh)
      || keep < 0 || (pb && sink))
    return TQ_ERR_BAD_ARG;
  if (hd % 16 != 0 || hd < 16 || hd > 512 || page_size % TILE != 0 || nkv <= 0 || nh % nkv != 0)
    return TQ_ERR_UNSUPPORTED;
  if (nh > 65535 || B > 65535 || page_stride % 8 != 0 || !(scale > 0.f)) return TQ_ERR_UNSUPPORTED;
  if (decode && most_runs(max_end) > MAX_RUNS_LDS) return TQ_ERR_UNSUPPORTED;
  AttnArgs a{(const bf16_t*)q, (const bf16_t*)k_pool, (const bf16_t*)v_pool, block_table, bt_stride, cu_seqlens, slots,
             start, page_size, page_stride, nh, nkv, hd, window, scale, (bf16_t*)out, partial,
             most_runs(max_end), ScoreMod{softcap, r1, r2, chunk, sink, pb, keep}, head_gate, ld_gate, ldo};
  const int dt = hd / 16;
  // head sizes 64, 128 and 256 have kernels of their own in which nothing depends on hd at run time
  if (decode) {
    if (!partial) return TQ_ERR_BAD_ARG;
    const int grid_runs = runs_at(max_end > 0 ? max_end - 1 : 0);      // the runs of the step's longest sequence
    if (dt == 4) launch_decode<4, true>(a, B, grid_runs, st);
    else if (dt == 8) launch_decode<8, true>(a, B, grid_runs, st);
    else if (dt == 16) launch_decode<16, true>(a, B, grid_runs, st);
    else if (dt < 4) launch_decode<4, false>(a, B, grid_runs, st);
    else if (dt < 8) launch_decode<8, false>(a, B, grid_runs, st);
    else if (dt < 16) launch_decode<16, false>(a, B, grid_runs, st);
    else if (dt == 32) launch_decode<32, true>(a, B, grid_runs, st);
    else launch_decode<32, false>(a, B, grid_runs, st);
  } else {
    // two groups of 16 tokens per wave, which halves the reads from LDS per product, when that still leaves
    // the chip two workgroups per compute unit and registers allow; else one group
    const bool two = (int64_t)((max_new + 127) / 128) * nh * B >= 512;
    int rc;
    if (dt == 4) rc = two ? launch_prefill<4, 2, true>(a, B, max_new, st) : launch_prefill<4, 1, true>(a, B, max_new, st);
    else if (dt == 8) rc = two ? launch_prefill<8, 2, true>(a, B, max_new, st) : launch_prefill<8, 1, true>(a, B, max_new, st);
    else if (dt == 16) rc = launch_prefill<16, 1, true>(a, B, max_new, st);
    // a head of 192 (128 plain and 64 rotated numbers of a latent attention's keys), with values of 128 or of 192
    else if (dt == 12 && value_width > 0 && value_width <= 128)
      rc = two ? launch_prefill<12, 2, true, 8>(a, B, max_new, st) : launch_prefill<12, 1, true, 8>(a, B, max_new, st);
    else if (dt == 12) rc = launch_prefill<12, 1, true>(a, B, max_new, st);
    else if (dt < 4) rc = two ? launch_prefill<4, 2, false>(a, B, max_new, st) : launch_prefill<4, 1, false>(a, B, max_new, st);
    else if (dt < 8) rc = two ? launch_prefill<8, 2, false>(a, B, max_new, st) : launch_prefill<8, 1, false>(a, B, max_new, st);
    else if (dt < 16) rc = launch_prefill<16, 1, false>(a, B, max_new, st);
    else if (dt == 32) rc = launch_prefill<32, 1, true>(a, B, max_new, st);
    else rc = launch_prefill<32, 1, false>(a, B, max_new, st);
    if (rc) return rc;
  }
  TQ_LAUNCH_CHECK();
  return 0;
}

TQ_API int tq_attention_mfma_sig(const void* q, const void* k_pool, const void* v_pool, const int* block_table,
                                       int bt_stride, const int* cu_seqlens, const int* slots, const int* start, int page_size,
                                       int64_t page_stride, int B, int nh, int nkv, int hd, int window, float scale,
                                       float softcap, const float* r1, const float* r2, int chunk, const float* sink,
                                       void* out, float* partial, int decode, int max_new, int max_end, int value_width,
                                       const float* head_gate, int64_t ld_gate, const float* pb, int keep, hipStream_t st) {
  return tq_attention_mfma_ld(q, k_pool, v_pool, block_table, bt_stride, cu_seqlens, slots, start, page_size, page_stride, B,
                              nh, nkv, hd, window, scale, softcap, r1, r2, chunk, sink, out, partial, decode, max_new, max_end,
                              value_width, head_gate, ld_gate, pb, keep, 0, st);
}

TQ_API int tq_attention_mfma_ex(const void* q, const void* k_pool, const void* v_pool, const int* block_table,
                                       int bt_stride, const int* cu_seqlens, const int* slots, const int* start, int page_size,
                                       int64_t page_stride, int B, int nh, int nkv, int hd, int window, float scale,
                                       float softcap, const float* r1, const float* r2, int chunk, const float* sink,
                                       void* out, float* partial, int decode, int max_new, int max_end, int value_width,
                                       const float* head_gate, int64_t ld_gate, hipStream_t st) {
  return tq_attention_mfma_sig(q, k_pool, v_pool, block_table, bt_stride, cu_seqlens, slots, start, page_size, page_stride, B,
                               nh, nkv, hd, window, scale, softcap, r1, r2, chunk, sink, out, partial, decode, max_new, max_end,
                               value_width, head_gate, ld_gate, nullptr, 0, st);
}

TQ_API int tq_attention_mfma_mod(const void* q, const void* k_pool, const void* v_pool, const int* block_table,
                                 int bt_stride, const int* cu_seqlens, const int* slots, const int* start, int page_size,
                                 int64_t page_stride, int B, int nh, int nkv, int hd, int window, float scale,
                                 float softcap, const float* r1, const float* r2, int chunk, const float* sink,
                                 void* out, float* partial, int decode, int max_new, int max_end, hipStream_t st) {
  return tq_attention_mfma_ex(q, k_pool, v_pool, block_table, bt_stride, cu_seqlens, slots, start, page_size,
                              page_stride, B, nh, nkv, hd, window, scale, softcap, r1, r2, chunk, sink, out, partial,
                              decode, max_new, max_end, 0, nullptr, 0, st);
}

TQ_API int tq_attention_mfma(const void* q, const void* k_pool, const void* v_pool, const int* block_table,
                             int bt_stride, const int* cu_seqlens, const int* slots, const int* start, int page_size,
                             int64_t page_stride, int B, int nh, int nkv, int hd, int window, float scale, void* out,
                             float* partial, int decode, int max_new, int max_end, hipStream_t st) {
  return tq_attention_mfma_mod(q, k_pool, v_pool, block_table, bt_stride, cu_seqlens, slots, start, page_size, page_stride,
                               B, nh, nkv, hd, window, scale, 0.f, nullptr, nullptr, 0, nullptr, out, partial, decode, max_new,
                               max_end, st);
}

// Differential attention over heads of hd (a multiple of 32, at most 256): a key row holds both maps' keys, each half of hd wide,
// a value row hd numbers of which the first vd count.  Prompts: q [T][nh][hd], both maps of a head side by side; decoding:
// q [T][2 nh][hd], each map alone with zeros in the other's place.  out [T][nh][hd] = r / sqrt(sum(r^2) / vd + eps) * post *
// sigmoid(gate), r = a1 - lambda a2; gate: float rows ld_gate apart, or null.  partial as tq_attention_decode_scratch says for 2 nh
// heads.
TQ_API int tq_attention_mfma_diff(const void* q, const void* k_pool, const void* v_pool, const int* block_table, int bt_stride,
                                  const int* cu_seqlens, const int* slots, const int* start, int page_size, int64_t page_stride,
                                  int B, int nh, int nkv, int hd, float scale, float lambda, float eps, int vd, float post,
                                  const float* gate, int64_t ld_gate, void* out, float* partial, int decode, int max_new,
                                  int max_end, hipStream_t st) {
  if (B <= 0) return 0;
  if (hd % 32 != 0 || hd < 32 || hd > 256 || page_size % TILE != 0 || nkv <= 0 || nh % nkv != 0) return TQ_ERR_UNSUPPORTED;
  if (nh > 32767 || B > 65535 || page_stride % 8 != 0 || !(scale > 0.f)) return TQ_ERR_UNSUPPORTED;
  if (vd < 1 || vd > hd || (gate && (ld_gate < (int64_t)nh * hd || ld_gate % 4 != 0 || (uintptr_t)gate % 16 != 0))) return TQ_ERR_BAD_ARG;
  if (decode && (!partial || most_runs(max_end) > MAX_RUNS_LDS)) return TQ_ERR_BAD_ARG;
  const DiffArgs df{lambda, eps, post, vd, gate, ld_gate};
  AttnArgs a{(const bf16_t*)q, (const bf16_t*)k_pool, (const bf16_t*)v_pool, block_table, bt_stride, cu_seqlens, slots,
             start, page_size, page_stride, decode ? 2 * nh : nh, nkv, hd, 0, scale, (bf16_t*)out, partial,
             most_runs(max_end), ScoreMod{}, nullptr, 0, (int64_t)nh * hd};
  const int dt = hd / 16;
  int rc = 0;
  if (decode) {
    const int grid_runs = runs_at(max_end > 0 ? max_end - 1 : 0);
    if (dt == 4) launch_decode_as<4, true, false>(a, B, grid_runs, st, &df);
    else if (dt == 8) launch_decode_as<8, true, false>(a, B, grid_runs, st, &df);
    else if (dt == 16) launch_decode_as<16, true, false>(a, B, grid_runs, st, &df);
    else if (dt < 4) launch_decode_as<4, false, false>(a, B, grid_runs, st, &df);
    else if (dt < 8) launch_decode_as<8, false, false>(a, B, grid_runs, st, &df);
    else launch_decode_as<16, false, false>(a, B, grid_runs, st, &df);
  } else {
    if (dt == 4) rc = launch_diff_prefill<4, true>(a, df, B, max_new, st);
    else if (dt == 8) rc = launch_diff_prefill<8, true>(a, df, B, max_new, st);
    else if (dt == 16) rc = launch_diff_prefill<16, true>(a, df, B, max_new, st);
    else if (dt < 4) rc = launch_diff_prefill<4, false>(a, df, B, max_new, st);
    else if (dt < 8) rc = launch_diff_prefill<8, false>(a, df, B, max_new, st);
    else rc = launch_diff_prefill<16, false>(a, df, B, max_new, st);
  }
  if (rc) return rc;
  TQ_LAUNCH_CHECK();
  return 0;
}
