// ixt_heads_kernels.h -- attention of hybrid decoders over keys and values per head (IXT_MIX_ATTENTION): query heads in equal groups on one key / value
// head each, optional norm of query and key heads, rotation of a head's first features, optional window, optional sink (a number per head that joins the
// softmax denominator without a key or a value), optional soft cap of the scores, optional gate on the concatenated heads.  Sizes of keys and values are
// independent.  Values may be the keys as projected; a chunked mask shows a position the keys of its own chunk only; the gate may be one number per head.
// With two maps a head has two queries and its key head two keys per token, both of `d` features, over the same values; the two outputs
// become one: a1 - lambda a2, over its root mean square, times a constant (differential attention).
//
//   k_heads_prep     projection slices -> queries [R][H][dkp], the row's keys and values in their pages
//   k_heads_prompt   many rows, bf16, matrix cores
//   k_heads_decode   few rows, bf16, matrix cores, keys split over blocks (+ k_heads_combine)
//   k_heads_any      any sizes, any T
//
// Pages: [page][kv head][token][dkp] (the maps dmp apart in a row) and [page][kv head][token][dvp]; what lies behind the real features is zero from the
// pool's creation on.
#pragma once
#include "ixt_hybrid_kernels.h"

struct HeadsGeom {
  int H, G, d, dv, rot, P, mpg, window;     // query heads, key / value heads, key and value dims, rotated dims, page size, pages per group, window (<= 0: none)
  int dkp, dvp;                             // padded key / value rows
  int maps, dmp;                            // softmax maps per head (1, 2); a map's part of a key row: dkp = maps dmp
  int hs, vs, ok, ov, og;                   // projection columns: a map of a query / key head takes hs, a value head vs; keys from ok on, values from ov on, gates
                                            // (vs per query head, or one: head_gate) from og on (< 0: none)
  float scale, cap;                         // cap > 0: score <- cap tanh(score / cap)
  int chunk, head_gate;                     // chunk > 0: only keys of the position's own chunk of that many positions (window unused)
  int oc, kend;                             // act of the output projection: the heads' first column, and where the zeros behind them end
  float of;                                 // factor on the outputs
};
// the first key that position p sees
__device__ __forceinline__ int first_key(const HeadsGeom& g, int p) { return g.chunk > 0 ? p - p % g.chunk : g.window > 0 ? max(0, p - g.window + 1) : 0; }
struct MapsArgs { const float* lambda; float keep, eps; };               // two maps: (a1 - *lambda a2) / rms(., eps) keep
struct RowsArgs { const int32_t *slot, *pos, *active, *page_map; };      // the rows of a pass

// A query or key head (columns c0 .. of row r of the projection) by LP lanes, four features each at a time: norm by w (nullptr: none), rotation;
// emit(f, o): features f .. f + 3 of the n asked for (zeros behind the head's own).  rope: f32 [position][rot / 2] cos, sin.
struct HeadsRope { const float *cos, *sin; };
template <int LP, typename G, typename F>
__device__ __forceinline__ void head_norm_rotate(const Slices& t, int r, int c0, const G& g, const float* __restrict__ w, float eps, HeadsRope rope, int pos, int n, int sl, F emit) {
  float v[4] = {0.0f, 0.0f, 0.0f, 0.0f}, rs = 1.0f;
  if (sl * 4 < g.hs) t.at4(r, c0 + sl * 4, v);              // (columns d .. hs - 1 are zero)
  if (w != nullptr) {
    float ss = fmaf(v[0], v[0], fmaf(v[1], v[1], fmaf(v[2], v[2], v[3] * v[3])));
    for (int f = (sl + LP) * 4; f < g.hs; f += 4 * LP) {
      float u[4];
      t.at4(r, c0 + f, u);
      ss += fmaf(u[0], u[0], fmaf(u[1], u[1], fmaf(u[2], u[2], u[3] * u[3])));
    }
    ss = row16_sum(ss);
#pragma unroll
    for (int off = 16; off < LP; off <<= 1) ss += __shfl_xor(ss, off, 64);
    rs = 1.0f / sqrtf(ss / (float)g.d + eps);
  }
  const int half = g.rot >> 1;
  for (int f = sl * 4; f < n; f += 4 * LP) {
    if (f != sl * 4) {
      v[0] = v[1] = v[2] = v[3] = 0.0f;
      if (f < g.hs) t.at4(r, c0 + f, v);
    }
    if (w != nullptr && f < g.hs) {                         // (the weight's tail is zero, too)
      const float4 ww = *reinterpret_cast<const float4*>(w + f);
      v[0] *= rs * ww.x; v[1] *= rs * ww.y; v[2] *= rs * ww.z; v[3] *= rs * ww.w;
    }
    float o[4] = {v[0], v[1], v[2], v[3]};
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int pr = f / 2 + i;
      if (pr < half) {
        const float c = rope.cos[(size_t)pos * half + pr], s = rope.sin[(size_t)pos * half + pr];
        o[2 * i] = v[2 * i] * c - v[2 * i + 1] * s;
        o[2 * i + 1] = v[2 * i + 1] * c + v[2 * i] * s;
      }
    }
    emit(f, o);
  }
}
// lambda = exp(lq1 . lk1) - exp(lq2 . lk2) + diff.  One wave.
static __global__ __launch_bounds__(64) void k_maps_lambda(const float* lq1, const float* lk1, const float* lq2, const float* lk2, int n, float diff, float* lambda) {
  float a = 0.0f, b = 0.0f;
  for (int i = threadIdx.x; i < n; i += 64) { a = fmaf(lq1[i], lk1[i], a); b = fmaf(lq2[i], lk2[i], b); }
  a = wave_sum(a); b = wave_sum(b);
  if (threadIdx.x == 0) *lambda = expf(a) - expf(b) + diff;
}
// four columns of the concatenated heads (c % 4 == 0 inside head h) times their gate and the layer's factor -> act
__device__ __forceinline__ void heads_out4(const Slices& t, int r, const HeadsGeom& g, int h, int c, float* v, bf16_t* out, int Kp) {
  if (g.og >= 0) {
    float z[4];
    if (g.head_gate) z[0] = z[1] = z[2] = z[3] = t.at(r, g.og + h);
    else t.at4(r, g.og + h * g.vs + c, z);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] *= hw_rcp(1.0f + hw_exp2(-1.44269504088896340736f * z[j]));
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] *= g.of;
  act_store4(out, r, g.oc + h * g.vs + c, Kp, v);
}
// log2(e) times the capped score, cap (1 - 2 / (1 + exp(2 s scale / cap))): c2 = 2 scale log2(e) / cap, k2 = cap log2(e)
__device__ __forceinline__ float capped_log2(float s, float c2, float k2) { return fmaf(-2.0f * k2, hw_rcp(1.0f + hw_exp2(c2 * s)), k2); }

// LP lanes per map of a head (16, 32, 64): queries [R][H][maps][dmp], and the row's keys and values in their pages.  grid (R, ceil((maps (H + G) + G) LP /
// 256)), block 256.
template <typename T, int LP>
__global__ __launch_bounds__(256) void k_heads_prep(Slices t, HeadsGeom g, const float* __restrict__ qn, const float* __restrict__ kn, float eps, HeadsRope rope, RowsArgs rows,
                                                    T* __restrict__ kpages, T* __restrict__ vpages, T* __restrict__ q) {
  const int r = blockIdx.x, j = blockIdx.y * (256 / LP) + threadIdx.x / LP, sl = threadIdx.x % LP, QU = g.H * g.maps, KU = g.G * g.maps;
  if (j >= QU + KU + g.G) return;
  const bool act = rows.active[r] != 0;
  if (!act && j >= QU) return;
  const int pos = act ? rows.pos[r] : 0;
  if (j < QU) {
    T* o = q + ((size_t)r * QU + j) * g.dmp;
    head_norm_rotate<LP>(t, r, j * g.hs, g, qn, eps, rope, pos, g.dmp, sl, [&](int f, const float* v) { store4(o + f, v); });
    return;
  }
  const int ku = j - QU, kh = ku < KU ? ku / g.maps : ku - KU;
  const size_t at = ((size_t)rows.page_map[(size_t)rows.slot[r] * g.mpg + pos / g.P] * g.G + kh) * g.P + pos % g.P;          // row of the key / value pools
  if (ku < KU) {
    T* o = kpages + at * g.dkp + ku % g.maps * g.dmp;
    head_norm_rotate<LP>(t, r, g.ok + ku * g.hs, g, kn, eps, rope, pos, g.hs, sl, [&](int f, const float* v) { store4(o + f, v); });
    return;
  }
  T* o = vpages + at * g.dvp;
  for (int f = sl * 4; f < g.vs; f += 4 * LP) {
    float v[4];
    t.at4(r, g.ov + kh * g.vs + f, v);
    store4(o + f, v);
  }
}

// Any sizes (dv <= 1024), any T: block = (row, head); thread = key for the scores (tiles of 256 keys, running maximum and sum, the sink as their start),
// thread = value column for the weighted sum; two maps one after the other.  t: the projection (gates).  out: act(T), column h vs + c.  grid (R, H), block
// 256, LDS = (dkp + 256) floats.
template <typename T>
__global__ __launch_bounds__(256) void k_heads_any(const T* __restrict__ qb, HeadsGeom g, const float* __restrict__ sink, RowsArgs rows, const T* __restrict__ kpages,
                                                   const T* __restrict__ vpages, MapsArgs mp, Slices t, T* __restrict__ out, int Kp) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[4];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, kh = h / (g.H / g.G);
  if (!rows.active[r]) return;
  float* q = sm;
  float* p = sm + g.dkp;
  for (int k = tid; k < g.dkp; k += 256) q[k] = to_f(qb[((size_t)r * g.H + h) * g.dkp + k]);
  __syncthreads();
  const int pos = rows.pos[r], k_lo = first_key(g, pos);
  const int32_t* prow = rows.page_map + (size_t)rows.slot[r] * g.mpg;
  float o[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int mi = 0; mi < g.maps; ++mi) {
    const float* qm = q + mi * g.dmp;
    float m = sink != nullptr ? sink[h] : -INFINITY, l = sink != nullptr ? 1.0f : 0.0f, acc[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int j0 = k_lo; j0 <= pos; j0 += 256) {
      const int j = j0 + tid;
      float s = -INFINITY;
      if (j <= pos) {
        const T* kp = kpages + (((size_t)prow[j / g.P] * g.G + kh) * g.P + j % g.P) * g.dkp + mi * g.dmp;
        float a = 0.0f;
        for (int k = 0; k < g.d; ++k) a = fmaf(qm[k], to_f(kp[k]), a);
        s = a * g.scale;
        if (g.cap > 0.0f) s = g.cap * tanhf(s / g.cap);
      }
      float tm = s;
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) tm = fmaxf(tm, __shfl_xor(tm, off, 64));
      __syncthreads();
      if ((tid & 63) == 0) red[tid >> 6] = tm;
      __syncthreads();
      const float mn = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m);
      const float e = j <= pos ? expf(s - mn) : 0.0f;
      p[tid] = e;
      const float al = expf(m - mn);
      const float ls = block_sum256(e, red);                  // (its barriers also publish p)
      l = l * al + ls;
      m = mn;
      const int nk = min(256, pos - j0 + 1);
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] *= al;
      for (int kk = 0; kk < nk; ++kk) {
        const T* vp = vpages + (((size_t)prow[(j0 + kk) / g.P] * g.G + kh) * g.P + (j0 + kk) % g.P) * g.dvp;
        const float w = p[kk];
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (tid + 256 * i < g.dv) acc[i] = fmaf(w, to_f(vp[tid + 256 * i]), acc[i]);
      }
      __syncthreads();
    }
    const float f = mi == 0 ? 1.0f / l : -*mp.lambda / l;
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = mi == 0 ? acc[i] / l : fmaf(acc[i], f, o[i]);
  }
  if (g.maps > 1) {
    float ss = 0.0f;                                        // (columns from dv on are zero)
#pragma unroll
    for (int i = 0; i < 4; ++i) ss = fmaf(o[i], o[i], ss);
    const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)g.dv + mp.eps) * mp.keep;
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] *= rs;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = tid + 256 * i;
    if (c >= g.vs) continue;
    if (g.og >= 0 && c < g.dv) o[i] *= f32_sigmoid(t.at(r, g.og + (g.head_gate ? h : h * g.vs + c)));
    act_store1(out, r, g.oc + h * g.vs + c, Kp, o[i] * g.of);
  }
  if (h == g.H - 1)
    for (int k = g.oc + g.H * g.vs + tid; k < g.kend; k += 256) act_store1(out, r, k, Kp, 0.0f);
}

// ---------------------------------------------------------------------------------------------------- matrix-core forms
// The M side of the products is (row, query head) pairs of one key / value head.  Per tile of 64 keys:
//   scores   D[key][pair] = mfma(A = keys, B = queries): a lane holds 4 keys of one pair per product
//   weights  running maximum / sum per pair in f32 (they start at the sink), exp2; P goes to bf16
//   output   D[column][pair] = mfma(A = values read column-wise, B = P)
// Two maps: pairs become (row, head, map) triples.
struct HeadsAttnArgs {
  const bf16_t* q; HeadsGeom g; const float* sink;
  RowsArgs rows;
  bf16_t *kpages, *vpages;
  int R, NQ, HB, hchunks, pshift;           // rows per block, query heads per block, blocks of query heads per key / value head
  bf16_t* out; int Kp;                      // act, column oc + h vs + c
  float *part_o, *part_ml;                  // splits > 1: [R H maps][splits][dvp], [R H maps][splits][2]
  Slices t; const float *qn, *kn; float eps; HeadsRope rope;      // the projection (gates); k_heads_decode with FUSED: and what k_heads_prep needs
  MapsArgs mp;
};
// the pool row of a key: page (G heads) -> head -> token
__device__ __forceinline__ int heads_row(const int32_t* __restrict__ prow, int key, int pshift, int G, int kh) {
  return ((prow[key >> pshift] * G + kh) << pshift) + (key & ((1 << pshift) - 1));
}

// Prompts: a block owns 64 pairs = up to 64 / HB consecutive rows x HB query heads of one key / value head (a wave 16 of them: 32 measured slower, 46
// against 29 us for 2048 rows of 16 heads); all waves walk the same key tiles, the next tile arriving while the current one is used.  P stays in registers: with the key order 4q .. 4q + 3, 16 + 4q ..
// 16 + 4q + 3 per lane group q of 32 keys, the lane's own scores ARE its operand of the next product.  Consecutive blocks are different heads: with
// 8 heads or a multiple of them, a head's keys and values stay in one XCD's L2.  grid (G hchunks, ceil(R / NQ)), block 256, LDS two tiles.
// MAPS 2: 32 (row, head) pairs; waves 0 and 1 take their first map, waves 2 and 3 the second (a wave needs one map's part of the keys), and hand its
// outputs over through LDS at the end.
template <int DK, int DV, int MAPS>
__global__ __launch_bounds__(256, DK + DV <= 320 ? 2 : 1) void k_heads_prompt(HeadsAttnArgs a) {
  static_assert(DK % (32 * MAPS) == 0, "whole steps per map");
  constexpr int NKS = DK / 32 / MAPS, NT = DV / 16, NGV = DV / 64, TILE = 64 * (DK + DV);
  extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
  const HeadsGeom& g = a.g;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r_in = lane & 15, cq = lane >> 4;
  const int kh = blockIdx.x % g.G, hc = blockIdx.x / g.G, GQ = g.H / g.G;
  const int r0 = blockIdx.y * a.NQ, nr = min(a.NQ, a.R - r0), h0 = kh * GQ + hc * a.HB, hb = min(a.HB, GQ - hc * a.HB);
  const int map = MAPS == 2 ? wave >> 1 : 0, pair = (MAPS == 2 ? wave & 1 : wave) * 16 + r_in, qi = pair / a.HB, hh = pair % a.HB;
  const bool pair_ok = qi < nr && hh < hb;
  const int row = r0 + (pair_ok ? qi : 0), head = h0 + (pair_ok ? hh : 0);
  const bool live = pair_ok && a.rows.active[row] != 0;
  const int pos = live ? a.rows.pos[row] : -1;
  bf16x8 qf[NKS];                                         // queries: lane = pair r_in, 8 consecutive features per step
#pragma unroll
  for (int ks = 0; ks < NKS; ++ks)
    qf[ks] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(a.q + (((size_t)row * g.H + head) * MAPS + map) * (DK / MAPS) + ks * 32 + cq * 8));
  float m = a.sink != nullptr ? a.sink[head] * 1.44269504088896340736f : -INFINITY, l = a.sink != nullptr ? 1.0f : 0.0f;
  f32x4 o[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) o[i] = f32x4(0.0f);
  const float sc = g.cap > 0.0f ? 1.0f : g.scale * 1.44269504088896340736f, c2 = g.cap > 0.0f ? 2.88539008177792681472f * g.scale / g.cap : 0.0f, k2 = g.cap * 1.44269504088896340736f;
  TileLane L = tile_lane(r_in, cq);
  if (map == 1) {                                         // the second map's keys lie NKS steps on in the row (NKS odd: its even steps are the odd ones of a group)
    const uint32_t k0 = L.k0;
    L.k0 = (NKS & 1 ? L.k1 : L.k0) + NKS / 2 * 8192;
    L.k1 = NKS & 1 ? k0 + (NKS / 2 + 1) * 8192 : L.k1 + NKS / 2 * 8192;
  }
  for (int ra = 0; ra < nr;) {                            // runs of rows that share a page group
    if (!a.rows.active[r0 + ra]) { ++ra; continue; }
    const int slot = a.rows.slot[r0 + ra];
    int lo = a.rows.pos[r0 + ra], hi = lo, rb = ra + 1;
    while (rb < nr && a.rows.active[r0 + rb] && a.rows.slot[r0 + rb] == slot) { const int p = a.rows.pos[r0 + rb]; lo = min(lo, p); hi = max(hi, p); ++rb; }
    const bool whole = ra == 0 && rb == nr;               // no other run in this block: only the keys decide what is masked
    const bool mine = live && qi >= ra && qi < rb;
    const int my_lo = mine ? first_key(g, pos) : 0;
    ra = rb;
    const int k_lo = first_key(g, lo), k_all = first_key(g, hi);      // (k_all .. lo: seen by every row)
    const int ntile = (hi - k_lo) / 64 + 1;
    const int32_t* prow = a.rows.page_map + (size_t)slot * g.mpg;
    __syncthreads();                                      // the previous run's last tile has been read
    int off = heads_row(prow, min(k_lo + lane, hi), a.pshift, g.G, kh);
    tile_dma<DK>(a.kpages, off, lds, wave, lane);
    tile_dma<DV>(a.vpages, off, lds + 64 * DK, wave, lane);
    off = heads_row(prow, min(k_lo + 64 + lane, hi), a.pshift, g.G, kh);
    for (int t = 0; t < ntile; ++t) {
      const bf16_t* tile = lds + (size_t)(t & 1) * TILE;
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      __syncthreads();                                    // the tile is there; every wave is done with the other one
      if (t + 1 < ntile) {
        bf16_t* next = lds + (size_t)((t + 1) & 1) * TILE;
        tile_dma<DK>(a.kpages, off, next, wave, lane);
        tile_dma<DV>(a.vpages, off, next + 64 * DK, wave, lane);
        off = heads_row(prow, min(k_lo + (t + 2) * 64 + lane, hi), a.pshift, g.G, kh);
      }
      f32x4 s[4];
#pragma unroll
      for (int n = 0; n < 4; ++n) s[n] = f32x4(0.0f);
      bf16x8 kf[2][4];                                    // operands one step ahead of the products
#pragma unroll
      for (int n = 0; n < 4; ++n) kf[0][n] = tile_kf<DK>(reinterpret_cast<const char*>(tile), L, 0, n);
#pragma unroll
      for (int ks = 0; ks < NKS; ++ks) {
        if (ks + 1 < NKS) {
#pragma unroll
          for (int n = 0; n < 4; ++n) kf[(ks + 1) & 1][n] = tile_kf<DK>(reinterpret_cast<const char*>(tile), L, ks + 1, n);
        }
#pragma unroll
        for (int n = 0; n < 4; ++n) s[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[ks & 1][n], qf[ks], s[n], 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0);
      }
      if (g.cap > 0.0f) {
#pragma unroll
        for (int n = 0; n < 4; ++n)
#pragma unroll
          for (int j = 0; j < 4; ++j) s[n][j] = capped_log2(s[n][j], c2, k2);
      }
      const int t0 = k_lo + t * 64;
      const bool inside = whole && t0 >= k_all && t0 + 63 <= lo;
      bf16x8 pf[2];
      float tm = -INFINITY;
      if (inside) {
#pragma unroll
        for (int n = 0; n < 4; ++n)
#pragma unroll
          for (int j = 0; j < 4; ++j) tm = fmaxf(tm, s[n][j]);
      } else {
#pragma unroll
        for (int n = 0; n < 4; ++n)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int key = t0 + n * 16 + cq * 4 + j;
            const bool seen = mine && key <= pos && key >= my_lo;
            s[n][j] = seen ? s[n][j] : -INFINITY;
            tm = fmaxf(tm, s[n][j]);
          }
      }
      tm *= sc;                                         // (a positive factor keeps the order)
      tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
      tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
      const float mn = fmaxf(m, tm), mz = mn == -INFINITY ? 0.0f : mn;
      const float al = hw_exp2(m - mz);           // (nothing seen so far: exp2(-inf) = 0, and l and o are 0)
      float ls = 0.0f;
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int j = 0; j < 4; ++j) { s[n][j] = hw_exp2(fmaf(s[n][j], sc, -mz)); ls += s[n][j]; }
      ls += __shfl_xor(ls, 16, 64);
      ls += __shfl_xor(ls, 32, 64);
      l = l * al + ls;
      m = mn;
      if (__any(al != 1.0f)) {
#pragma unroll
        for (int i = 0; i < NT; ++i) { o[i][0] *= al; o[i][1] *= al; o[i][2] *= al; o[i][3] *= al; }
      }
#pragma unroll
      for (int u = 0; u < 2; ++u) {                     // 32 keys each
        u32x4 pk;
        pk.x = pack2(f2bf(s[2 * u][0]), f2bf(s[2 * u][1])); pk.y = pack2(f2bf(s[2 * u][2]), f2bf(s[2 * u][3]));
        pk.z = pack2(f2bf(s[2 * u + 1][0]), f2bf(s[2 * u + 1][1])); pk.w = pack2(f2bf(s[2 * u + 1][2]), f2bf(s[2 * u + 1][3]));
        pf[u] = __builtin_bit_cast(bf16x8, pk);
      }
      const uint32_t tb = lds_addr(tile) + 64 * DK * 2;
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        [[maybe_unused]] uint2 f[2][4][2];
        if constexpr (NGV > 0) IXT_TILE_VT(f[0], tb, L, 0, u);
#pragma unroll
        for (int gr = 0; gr < NGV; ++gr) {                // the next group's reads travel under this one's products
          if (gr + 1 < NGV) {
            IXT_TILE_VT(f[(gr + 1) & 1], tb, L, gr + 1, u);
            IXT_TILE_VWAIT(f[gr & 1], 8);
          } else {
            IXT_TILE_VWAIT(f[gr & 1], 0);
          }
#pragma unroll
          for (int i = 0; i < 4; ++i) o[gr * 4 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tile_vfrag(f[gr & 1][i]), pf[u], o[gr * 4 + i], 0, 0, 0);
        }
        if constexpr (DV % 64 != 0) {
          uint2 fh[2][2];
          IXT_TILE_VTH(fh, tb, L, NGV, u);
          IXT_TILE_VWAITN(fh, 2, 0);
#pragma unroll
          for (int i = 0; i < 2; ++i) o[NGV * 4 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tile_vfrag(fh[i]), pf[u], o[NGV * 4 + i], 0, 0, 0);
        }
      }
    }
  }
  float inv = 1.0f / l;
  if constexpr (MAPS == 2) {
    f32x4* hand = reinterpret_cast<f32x4*>(lds);          // [wave & 1][column tile][lane]
    __syncthreads();                                      // the last tile has been read
    if (map == 1) {
#pragma unroll
      for (int i = 0; i < NT; ++i) hand[((wave & 1) * NT + i) * 64 + lane] = o[i] * inv;
    }
    __syncthreads();
    if (map == 1) return;
    const float lambda = *a.mp.lambda;
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const f32x4 o2 = hand[(wave * NT + i) * 64 + lane];
#pragma unroll
      for (int j = 0; j < 4; ++j) { o[i][j] = fmaf(-lambda, o2[j], o[i][j] * inv); ss = fmaf(o[i][j], o[i][j], ss); }
    }
    ss += __shfl_xor(ss, 16, 64);
    ss += __shfl_xor(ss, 32, 64);
    inv = a.mp.keep / sqrtf(ss / (float)g.dv + a.mp.eps);
  }
  if (!live) return;
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    float v[4] = {o[i][0] * inv, o[i][1] * inv, o[i][2] * inv, o[i][3] * inv};
    if (i * 16 + cq * 4 >= g.vs) continue;
    heads_out4(a.t, row, g, head, i * 16 + cq * 4, v, a.out, a.Kp);      // (columns dv .. vs - 1 are zero: so are the values there)
  }
  const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  if (head == g.H - 1)
    for (int c = g.oc + g.H * g.vs + cq * 4; c < g.kend; c += 16) act_store4(a.out, row, c, a.Kp, z);
}

// Few rows (decode): a block owns up to 16 query heads of one key / value head of ONE row and every gridDim.z-th key tile of its window.  Scores: a wave
// takes 16 of the 64 keys; P and the tile maxima meet in LDS; output: a wave takes every fourth column tile.  One tile of LDS: several blocks share a
// CU and one's loads run under the other's products.  grid (R, G hchunks, splits), block 256.
// FUSED (every row the only one of its page group): no k_heads_prep in front.  A block takes its queries from the projection while the first tile is on
// its way; the block with the last tile also takes the row's key and value, keeps them for later passes in their pages and puts them into its tile.
// MAPS 2: neighbouring pairs are the two maps of a head; a pair's query is zero on the other map's part of the keys.
template <int DK, int DV, bool FUSED, int MAPS>
__device__ __forceinline__ void heads_decode(const HeadsAttnArgs& a, const int row, const int hblock, const int split, const int nsplit, bf16_t* tile) {
  static_assert(DK % (32 * MAPS) == 0, "whole steps per map");
  constexpr int DM = DK / MAPS, NKM = DM / 32, NKS = DK / 32, NGV = DV / 64, NH = DV % 64 != 0 ? 1 : 0, OT = NGV + NH;     // column tiles per wave: one of every full group, waves 0 and 1 one of the half group
  __shared__ __attribute__((aligned(16))) bf16_t ps[16][72];
  __shared__ float s_m[4][16], s_l[4][16];
  __shared__ __attribute__((aligned(16))) bf16_t s_q[FUSED ? 16 : 1][DM + 8], s_k[FUSED ? DK : 8], s_v[FUSED ? DV : 8];
  const HeadsGeom& g = a.g;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r_in = lane & 15, cq = lane >> 4;
  const int kh = hblock % g.G, hc = hblock / g.G, GQ = g.H / g.G;
  const int h0 = kh * GQ + hc * a.HB, hb = min(a.HB, GQ - hc * a.HB), nu = hb * MAPS;
  const int active = a.rows.active[row], pos = a.rows.pos[row], slot = a.rows.slot[row];     // (requested together)
  if (!active) return;
  const bool pair_ok = r_in < nu;
  const int u_in = pair_ok ? r_in : 0, map = u_in % MAPS, head = h0 + u_in / MAPS;
  const int32_t* prow = a.rows.page_map + (size_t)slot * g.mpg;
  const int k_lo = first_key(g, pos), ntile = (pos - k_lo) / 64 + 1;
  int t = split;
  if (t < ntile) {
    const int off = heads_row(prow, min(k_lo + t * 64 + lane, pos), a.pshift, g.G, kh);
    tile_dma<DK>(a.kpages, off, tile, wave, lane);
    tile_dma<DV>(a.vpages, off, tile + 64 * DK, wave, lane);
  }
  bf16x8 qf[NKS];
  [[maybe_unused]] const bool last = (ntile - 1) % nsplit == split;       // the row's own key is in one of this block's tiles
  if constexpr (FUSED) {
    const size_t at = ((size_t)prow[pos >> a.pshift] * g.G + kh) * g.P + (pos & (g.P - 1));
    for (int i = wave; i < nu + (last ? MAPS + 1 : 0); i += 4) {
      if (i < nu) {
        head_norm_rotate<64>(a.t, row, (h0 * MAPS + i) * g.hs, g, a.qn, a.eps, a.rope, pos, DM, lane, [&](int f, const float* v) { store4(&s_q[i][f], v); });
      } else if (i < nu + MAPS) {
        const int m_ = i - nu;
        head_norm_rotate<64>(a.t, row, g.ok + (kh * MAPS + m_) * g.hs, g, a.kn, a.eps, a.rope, pos, DM, lane, [&](int f, const float* v) {
          store4(&s_k[m_ * DM + f], v);
          if (hc == 0 && f < g.hs) store4(a.kpages + at * DK + m_ * DM + f, v);
        });
      } else if (lane * 4 < DV) {
        float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
        if (lane * 4 < g.vs) a.t.at4(row, g.ov + kh * g.vs + lane * 4, v);
        store4(&s_v[lane * 4], v);
        if (hc == 0 && lane * 4 < g.vs) store4(a.vpages + at * DV + lane * 4, v);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int ks = 0; ks < NKS; ++ks) {
    const int km = ks % NKM * 32 + cq * 8;
    const u32x4 v = *reinterpret_cast<const u32x4*>(FUSED ? &s_q[u_in][km] : a.q + (((size_t)row * g.H + head) * MAPS + map) * DM + km);
    qf[ks] = __builtin_bit_cast(bf16x8, MAPS == 1 || ks / NKM == map ? v : u32x4(0));
  }
  f32x4 o[OT];
#pragma unroll
  for (int i = 0; i < OT; ++i) o[i] = f32x4(0.0f);
  const bool sink = a.sink != nullptr && split == 0;          // counted once
  float m = sink ? a.sink[head] * 1.44269504088896340736f : -INFINITY, l = sink && wave == 0 && cq == 0 ? 1.0f : 0.0f;      // l: this lane's keys only
  const float sc = g.scale * 1.44269504088896340736f, c2 = g.cap > 0.0f ? 2.88539008177792681472f * g.scale / g.cap : 0.0f, k2 = g.cap * 1.44269504088896340736f;
  const TileLane L = tile_lane(r_in, cq);
  const uint32_t vl = wave == 0 ? L.v[0] : (wave == 1 ? L.v[1] : (wave == 2 ? L.v[2] : L.v[3]));
  [[maybe_unused]] const uint32_t vh = (wave & 1) ? L.vh[1] : L.vh[0];
  const uint32_t tb = lds_addr(tile) + 64 * DK * 2;
  for (; t < ntile; t += nsplit) {
    int off = 0;
    if (t + nsplit < ntile) off = heads_row(prow, min(k_lo + (t + nsplit) * 64 + lane, pos), a.pshift, g.G, kh);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (FUSED && last && t == ntile - 1) {                // over what the tile's load found in the page
      const int rr = pos - k_lo - t * 64;
      if (tid < DK / 8) tile_put<DK>(tile, rr, tid, *reinterpret_cast<const u32x4*>(&s_k[tid * 8]));
      else if (tid >= 64 && tid < 64 + DV / 8) tile_put<DV>(tile + 64 * DK, rr, tid - 64, *reinterpret_cast<const u32x4*>(&s_v[(tid - 64) * 8]));
      __syncthreads();
    }
    f32x4 s = f32x4(0.0f);
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks)
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tile_kf<DK>(reinterpret_cast<const char*>(tile) + wave * (DK % 64 != 0 && ks == DK / 64 * 2 ? 1024 : 2048), L, ks, 0), qf[ks], s, 0, 0, 0);
    float tm = -INFINITY;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      s[j] = k_lo + t * 64 + wave * 16 + cq * 4 + j <= pos ? (g.cap > 0.0f ? capped_log2(s[j], c2, k2) : s[j] * sc) : -INFINITY;
      tm = fmaxf(tm, s[j]);
    }
    tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
    tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
    if (cq == 0) s_m[wave][r_in] = tm;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(s_m[0][r_in], s_m[1][r_in]), fmaxf(s_m[2][r_in], s_m[3][r_in])));   // (a tile has at least one visible key: finite)
    const float al = hw_exp2(m - mn);
    float p[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) p[j] = hw_exp2(s[j] - mn);
    l = l * al + ((p[0] + p[1]) + (p[2] + p[3]));
    m = mn;
    uint2 pk;
    pk.x = pack2(f2bf(p[0]), f2bf(p[1])); pk.y = pack2(f2bf(p[2]), f2bf(p[3]));
    *reinterpret_cast<uint2*>(&ps[r_in][wave * 16 + cq * 4]) = pk;
    if (__any(al != 1.0f)) {
#pragma unroll
      for (int i = 0; i < OT; ++i) { o[i][0] *= al; o[i][1] *= al; o[i][2] *= al; o[i][3] *= al; }
    }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 2; ++u) {                         // lane group q holds keys 32 u + 4 q .. + 3 and 32 u + 16 + 4 q .. + 3 (as in k_heads_prompt)
      uint2 f[OT][2];
#pragma unroll
      for (int i = 0; i < NGV; ++i) {
        asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(f[i][0]) : "v"(tb + vl), "n"(i * 8192 + u * 4096) : "memory");
        asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(f[i][1]) : "v"(tb + vl), "n"(i * 8192 + u * 4096 + 2048) : "memory");
      }
      if constexpr (NH == 1) {
        asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(f[NGV][0]) : "v"(tb + vh), "n"(NGV * 8192 + u * 2048) : "memory");
        asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(f[NGV][1]) : "v"(tb + vh), "n"(NGV * 8192 + u * 2048 + 1024) : "memory");
      }
      const uint2 p0 = *reinterpret_cast<const uint2*>(&ps[r_in][u * 32 + 4 * cq]), p1 = *reinterpret_cast<const uint2*>(&ps[r_in][u * 32 + 16 + 4 * cq]);
      u32x4 pv; pv.x = p0.x; pv.y = p0.y; pv.z = p1.x; pv.w = p1.y;
      const bf16x8 pf = __builtin_bit_cast(bf16x8, pv);
      IXT_TILE_VWAITN(f, OT, 0);
#pragma unroll
      for (int i = 0; i < OT; ++i) o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tile_vfrag(f[i]), pf, o[i], 0, 0, 0);
    }
    __syncthreads();                                      // the tile has been read by every wave
    if (t + nsplit < ntile) {
      tile_dma<DK>(a.kpages, off, tile, wave, lane);
      tile_dma<DV>(a.vpages, off, tile + 64 * DK, wave, lane);
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (cq == 0) s_l[wave][r_in] = l;
  __syncthreads();
  l = (s_l[0][r_in] + s_l[1][r_in]) + (s_l[2][r_in] + s_l[3][r_in]);
  float inv = nsplit == 1 ? 1.0f / l : 1.0f;
  if (MAPS == 2 && nsplit == 1) {                         // the even pair of a head takes both
    const float lambda = *a.mp.lambda;
    float ss = 0.0f;
#pragma unroll
    for (int i = 0; i < OT; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float v = o[i][j] * inv;
        o[i][j] = fmaf(-lambda, __shfl_xor(v, 1, 64), v);
        if (i < NGV || wave <= 1) ss = fmaf(o[i][j], o[i][j], ss);
      }
    ss += __shfl_xor(ss, 16, 64);
    ss += __shfl_xor(ss, 32, 64);
    if (cq == 0) s_m[wave][r_in] = ss;
    __syncthreads();
    inv = a.mp.keep / sqrtf(((s_m[0][r_in] + s_m[1][r_in]) + (s_m[2][r_in] + s_m[3][r_in])) / (float)g.dv + a.mp.eps);
    if (map == 1) return;
  }
  if (!pair_ok) return;
  const size_t pi = (((size_t)row * g.H + head) * MAPS + map) * nsplit + split;
#pragma unroll
  for (int i = 0; i < OT; ++i) {
    if (i == NGV && wave > 1) continue;                   // the half group has two column tiles
    const int c = i * 64 + wave * 16 + cq * 4;
    float v[4] = {o[i][0] * inv, o[i][1] * inv, o[i][2] * inv, o[i][3] * inv};
    if (nsplit == 1) {
      if (c >= g.vs) continue;
      heads_out4(a.t, row, g, head, c, v, a.out, a.Kp);
    } else *reinterpret_cast<float4*>(a.part_o + pi * DV + c) = make_float4(v[0], v[1], v[2], v[3]);
  }
  if (nsplit > 1) {
    if (wave == 0 && cq == 0) { a.part_ml[pi * 2] = m; a.part_ml[pi * 2 + 1] = l; }
  } else if (head == g.H - 1 && wave == 0) {
    const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int c = g.oc + g.H * g.vs + cq * 4; c < g.kend; c += 16) act_store4(a.out, row, c, a.Kp, z);
  }
}
template <int DK, int DV, bool FUSED, int MAPS>
__global__ __launch_bounds__(256, 2) void k_heads_decode(HeadsAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) bf16_t tile[];
  heads_decode<DK, DV, FUSED, MAPS>(a, blockIdx.x, blockIdx.y, blockIdx.z, gridDim.z, tile);
}
// the key splits of one head of a row (and its maps) put together, by the first 64 threads or more of a block; nsplit <= 16, vs <= 256.
__device__ __forceinline__ void heads_combine(const float* __restrict__ part_o, const float* __restrict__ part_ml, int nsplit, const HeadsGeom& g, const MapsArgs& mp, const Slices& t,
                                              const int32_t* __restrict__ row_active, bf16_t* __restrict__ out, int Kp, int r, int h) {
  __shared__ float fac[2][16];
  const int tid = threadIdx.x, c = tid * 4, H = g.H, vs = g.vs, dvp = g.dvp;
  if (!row_active[r]) return;
  const size_t p0 = ((size_t)r * H + h) * g.maps * nsplit;
  for (int m = 0; m < g.maps; ++m) split_factors(part_ml + (p0 + m * nsplit) * 2, nsplit, tid, fac[m]);
  float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  if (c < vs) split_sum4(part_o + p0 * dvp + c, dvp, nsplit, fac[0], v);
  if (g.maps == 2) {
    const float lambda = *mp.lambda;
    float u[4] = {0.0f, 0.0f, 0.0f, 0.0f}, ss = 0.0f;
    if (c < vs) split_sum4(part_o + (p0 + nsplit) * dvp + c, dvp, nsplit, fac[1], u);
#pragma unroll
    for (int j = 0; j < 4; ++j) { v[j] = fmaf(-lambda, u[j], v[j]); ss = fmaf(v[j], v[j], ss); }
    const float rs = mp.keep / sqrtf(wave_sum(ss) / (float)g.dv + mp.eps);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] *= rs;
  }
  if (c < vs) heads_out4(t, r, g, h, c, v, out, Kp);
  const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  if (h == H - 1)
    for (int c = g.oc + H * vs + tid * 4; c < g.kend; c += blockDim.x * 4) act_store4(out, r, c, Kp, z);
}
// grid (R, H), block 64
static __global__ __launch_bounds__(64) void k_heads_combine(const float* __restrict__ part_o, const float* __restrict__ part_ml, int nsplit, HeadsGeom g, MapsArgs mp, Slices t,
                                                      const int32_t* __restrict__ row_active, bf16_t* __restrict__ out, int Kp) {
  heads_combine(part_o, part_ml, nsplit, g, mp, t, row_active, out, Kp, blockIdx.x, blockIdx.y);
}
