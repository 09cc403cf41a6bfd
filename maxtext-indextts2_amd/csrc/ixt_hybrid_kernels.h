// ixt_hybrid_kernels.h -- kernels of decoders whose layers are listed one by one (ixt_config.layers): each layer has a sequence mixer (latent
// attention over a paged latent cache, a gated delta rule with a recurrent state per page group, attention over keys and values per head:
// ixt_heads_kernels.h, retention and lightning attention: ixt_retention_kernels.h, selective scan: ixt_scan_kernels.h), a feed-forward (a unit, dense or as a routed mixture) and norms in front of the sublayers,
// behind them, or both (in front of a mixer also a shift towards the token before); around a sublayer stands one residual sum, or several streams that mix
// (hyper-connections).
//
// Every kernel is a template over T, the storage of activations and cached keys: bf16_t (activations in the dot kernels' fragment order, xidx) or
// float (row-major; the 32-bit mode).  The residual stream, norms, rotations, scores, routers and the recurrence are f32 in both.
//
//   act(T)      an activation matrix [rows][Kp], Kp a multiple of 128 with zeros behind the real columns, in the order the dot of T reads
//   "slices"    a dot's output: f32 [slices][rows][ncols], to be added up by the reader
#pragma once
#include "ixt_kernels.h"
#include "ixt_moe_kernels.h"

// ---------------------------------------------------------------------------------------------------- activation storage
__device__ __forceinline__ void act_store1(bf16_t* b, int r, int k, int Kp, float v) { b[xidx(r, k, Kp)] = f2bf(v); }
__device__ __forceinline__ void act_store1(float* b, int r, int k, int Kp, float v) { b[(size_t)r * Kp + k] = v; }
template <typename T> __device__ __forceinline__ size_t act_at(int r, int k, int Kp) { return sizeof(T) == 2 ? (size_t)xidx(r, k, Kp) : (size_t)r * Kp + k; }      // place of an element
__device__ __forceinline__ void act_store4(bf16_t* b, int r, int k0, int Kp, const float* v) {      // k0 % 4 == 0
  uint2 o;
  o.x = pack2(f2bf(v[0]), f2bf(v[1])); o.y = pack2(f2bf(v[2]), f2bf(v[3]));
  *reinterpret_cast<uint2*>(b + xidx(r, k0, Kp)) = o;
}
__device__ __forceinline__ void act_store4(float* b, int r, int k0, int Kp, const float* v) {
  *reinterpret_cast<float4*>(b + (size_t)r * Kp + k0) = make_float4(v[0], v[1], v[2], v[3]);
}
__device__ __forceinline__ void act_store8(bf16_t* b, int r, int k0, int Kp, const float* v) {      // k0 % 8 == 0
  u32x4 o;
  o.x = pack2(f2bf(v[0]), f2bf(v[1])); o.y = pack2(f2bf(v[2]), f2bf(v[3])); o.z = pack2(f2bf(v[4]), f2bf(v[5])); o.w = pack2(f2bf(v[6]), f2bf(v[7]));
  *reinterpret_cast<u32x4*>(b + xidx(r, k0, Kp)) = o;
}
__device__ __forceinline__ void act_store8(float* b, int r, int k0, int Kp, const float* v) {
  act_store4(b, r, k0, Kp, v); act_store4(b, r, k0 + 4, Kp, v + 4);
}
__device__ __forceinline__ float to_f(bf16_t v) { return bf2f(v); }
__device__ __forceinline__ float to_f(float v) { return v; }
template <typename T> __device__ __forceinline__ T from_f(float v);
template <> __device__ __forceinline__ bf16_t from_f<bf16_t>(float v) { return f2bf(v); }
template <> __device__ __forceinline__ float from_f<float>(float v) { return v; }

struct Slices {             // a dot's output; bias: one number per column joins the sum (nullptr: none)
  const float* p; int n; size_t stride; int ncols; const float* bias = nullptr;
  __device__ __forceinline__ float at(int r, int c) const {
    const float* q = p + (size_t)r * ncols + c;
    float t = q[0];
    for (int s = 1; s < n; ++s) t += q[(size_t)s * stride];
    if (bias != nullptr) t += bias[c];
    return t;
  }
  template <int B = 4>
  __device__ __forceinline__ void at4(int r, int c, float* o) const {       // c % 4 == 0; B slices in flight
    const float* q = p + (size_t)r * ncols + c;
    float4 t = *reinterpret_cast<const float4*>(q);
    for (int s = 1; s < n; s += B) {
      float4 u[B];
#pragma unroll
      for (int i = 0; i < B; ++i) u[i] = *reinterpret_cast<const float4*>(q + (size_t)min(s + i, n - 1) * stride);
#pragma unroll
      for (int i = 0; i < B; ++i)
        if (s + i < n) { t.x += u[i].x; t.y += u[i].y; t.z += u[i].z; t.w += u[i].w; }
    }
    if (bias != nullptr) {
      const float4 b = *reinterpret_cast<const float4*>(bias + c);
      t.x += b.x; t.y += b.y; t.z += b.z; t.w += b.w;
    }
    o[0] = t.x; o[1] = t.y; o[2] = t.z; o[3] = t.w;
  }
  // the columns from c on (c % 4 == 0)
  __host__ __device__ __forceinline__ Slices from(int c) const { Slices s = *this; s.p += c; if (bias != nullptr) s.bias += c; return s; }
};

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) v += __shfl_xor(v, off, 64);
  return v;
}
// sum over the 16 lanes of a DPP row, every lane ends up with it
__device__ __forceinline__ float row16_sum(float v) {
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x128, 0xf, 0xf, false));   // row_ror:8
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x124, 0xf, 0xf, false));   // row_ror:4
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x122, 0xf, 0xf, false));   // row_ror:2
  v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x121, 0xf, 0xf, false));   // row_ror:1
  return v;
}
__device__ __forceinline__ float block_sum256(float v, float* red /*[4] LDS*/) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}
__device__ __forceinline__ float f32_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float f32_softplus(float z) { return z > 20.0f ? z : log1pf(expf(z)); }
// The same by max(z, 0) + log(1 + e), e = exp(-|z|), log(1 + e) = 2 artanh(s), s = e / (2 + e) <= 1/3, by its series (next term below 2e-8 of the sum): error
// below 1e-6 of the value for |z| < 10, |z| 1e-7 beyond
__device__ __forceinline__ float hw_softplus(float z) {
  const float e = hw_exp2(-1.44269504088896340736f * fabsf(z)), s = e * hw_rcp(2.0f + e), q = s * s;
  float p = fmaf(q, 1.0f / 15.0f, 1.0f / 13.0f);
  p = fmaf(q, p, 1.0f / 11.0f); p = fmaf(q, p, 1.0f / 9.0f); p = fmaf(q, p, 1.0f / 7.0f); p = fmaf(q, p, 0.2f); p = fmaf(q, p, 1.0f / 3.0f);
  return fmaxf(z, 0.0f) + fmaf(2.0f * s * q, p, 2.0f * s);
}

// ---------------------------------------------------------------------------------------------------- f32 dot
// out[r][n] = sum_k x[r][k] w[n][k], k ascending by fma.  x [R][Kp], w [Np][Kp] row-major f32, Kp % 32 == 0, Np % 16 == 0.  Grouped: 16-row block rb
// uses the matrix of group rb_exp[rb] (-1: none), wstride floats apart.  grid (ceil(Np / 64), ceil(R / 16)), block 256 (16 rows x 16 column lanes).
static __global__ __launch_bounds__(256) void k_dot32(const float* __restrict__ x, const float* __restrict__ w, int Kp, int Np, int R, float* __restrict__ out,
                                               const int32_t* __restrict__ rb_exp, size_t wstride) {
  __shared__ float xs[16][33], ws[64][33];
  const int tid = threadIdx.x, n0 = blockIdx.x * 64, r0 = blockIdx.y * 16;
  if (rb_exp != nullptr) {
    const int ex = rb_exp[blockIdx.y];
    if (ex < 0) return;
    w += (size_t)ex * wstride;
  }
  const int tr = tid >> 4, tc = tid & 15;
  float acc[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int k0 = 0; k0 < Kp; k0 += 32) {
    for (int i = tid; i < 16 * 32; i += 256) xs[i >> 5][i & 31] = (r0 + (i >> 5) < R) ? x[(size_t)(r0 + (i >> 5)) * Kp + k0 + (i & 31)] : 0.0f;
    for (int i = tid; i < 64 * 32; i += 256) ws[i >> 5][i & 31] = (n0 + (i >> 5) < Np) ? w[(size_t)(n0 + (i >> 5)) * Kp + k0 + (i & 31)] : 0.0f;
    __syncthreads();
#pragma unroll 8
    for (int k = 0; k < 32; ++k) {
      const float xv = xs[tr][k];
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j] = fmaf(xv, ws[tc + 16 * j][k], acc[j]);
    }
    __syncthreads();
  }
  if (r0 + tr < R) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (n0 + tc + 16 * j < Np) out[(size_t)(r0 + tr) * Np + n0 + tc + 16 * j] = acc[j];
  }
}

// ---------------------------------------------------------------------------------------------------- weights
// src [n][k] row-major ([out, in] linear weights, rows `ld` apart) -> rows n of a dot operand of Kp k-columns, at (column n_off + n, k k_off + k).
// inter: 16-column tile j goes to tile 2 j + n_off (the two matrices of a gated unit side by side).  trans: src is [k][n].  ng / kg > 0: groups of ng
// columns (kg k) are laid ngp (kgp) apart, zeros between them.  rn > 0: of every rg columns those from r0 on are rn rotated features in halves (i turns
// with i + rn / 2); they are laid as neighbours, which is the order the kernels turn (the order of a head's features changes no score).  krn > 0: the same for
// the first krn of every krg inputs (values that are keys come in that order).
struct LoadMap { int n, k, ld, Kp, n_off, k_off, inter, trans, ng, ngp, kg, kgp, rg, r0, rn, krg, krn; };
__device__ __forceinline__ int halves_to_pairs(int i, int group, int first, int n) {
  const int f = i % group - first, h = n / 2;
  return f >= 0 && f < n ? i + (f < h ? 2 * f : 2 * (f - h) + 1) - f : i;
}
template <typename S, typename T>
__global__ void k_load_nk(const S* __restrict__ src, T* __restrict__ dst, LoadMap m) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= (int64_t)m.n * m.k) return;
  int nn = m.trans ? (int)(i % m.n) : (int)(i / m.k), kk = m.trans ? (int)(i / m.n) : (int)(i % m.k);
  const float v = to_f(src[m.trans ? (size_t)kk * m.ld + nn : (size_t)nn * m.ld + kk]);
  if (m.rn > 0) nn = halves_to_pairs(nn, m.rg, m.r0, m.rn);
  if (m.krn > 0) kk = halves_to_pairs(kk, m.krg, 0, m.krn);
  if (m.ng > 0) nn = nn / m.ng * m.ngp + nn % m.ng;
  if (m.kg > 0) kk = kk / m.kg * m.kgp + kk % m.kg;
  const int col = m.inter ? ((nn >> 4) * 2 + m.n_off) * 16 + (nn & 15) : m.n_off + nn;
  if constexpr (sizeof(T) == 2) dst[widx(m.k_off + kk, col, m.Kp)] = f2bf(v);
  else dst[(size_t)col * m.Kp + m.k_off + kk] = v;
}
template <typename S, typename T>
__global__ void k_load_rows(const S* __restrict__ src, T* __restrict__ dst, int64_t n, int64_t k, int64_t kp) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n * k) dst[i / k * kp + i % k] = from_f<T>(to_f(src[i]));
}
template <typename S, typename T>
__global__ void k_load_vec(const S* __restrict__ src, T* __restrict__ dst, int64_t n) {
  const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) dst[i] = from_f<T>(to_f(src[i]));
}

// ---------------------------------------------------------------------------------------------------- row segments
// A segment = consecutive rows of one page group at consecutive positions: what a recurrence walks through.  One block of 1024 threads.
//   row_seg[r], row_j[r]   segment of row r and its place in it (row_seg -1: idle)
//   seg[s] = {first row, rows, page group, first position, parity of the convolution tail to read, first chunk, 0, 0}
//   chunk[c] = {first row, rows (<= SEG_CHUNK), segment, place in the segment}: a segment's chunks lie side by side (what a recurrence over blocks of
//   rows walks through), nseg_out[1] of them
// recurrent != 0: a segment must start at position 0 (the state counts as zero) or where its group's state stands (state_len); anything else, and a
// second segment of a group in one call, idles and is counted in err[0].  The tails of short convolutions are double-buffered: a pass reads parity
// p and writes 1 - p, so no row waits for another one's tail.
// head_rb: 16-row block b of a head-major activation matrix (rbh blocks per head) belongs to head b / rbh.
#define SEG_CHUNK 64
static __global__ __launch_bounds__(1024) void k_segments(int R, int32_t* row_active, const int32_t* row_slot, const int32_t* row_pos, int32_t* row_seg, int32_t* row_j,
                                                   int32_t* seg /*[.][8]*/, int4* chunk, int32_t* nseg_out, int32_t* state_len, int32_t* parity, int32_t* claim, int groups,
                                                   int recurrent, int32_t* err, int32_t* head_rb, int nhead_rb, int rbh) {
  __shared__ int s_last[1024];
  __shared__ int s_cnt, s_chunks;
  const int tid = threadIdx.x;
  for (int i = tid; i < groups; i += 1024) claim[i] = 0;
  for (int i = tid; i < nhead_rb; i += 1024) head_rb[i] = i / rbh;
  if (tid == 0) s_cnt = s_chunks = 0;
  const int per = (R + 1023) / 1024, lo = min(tid * per, R), hi = min(lo + per, R);
  auto starts = [&](int r) { return r == 0 || !row_active[r - 1] || row_slot[r - 1] != row_slot[r] || row_pos[r - 1] + 1 != row_pos[r]; };
  int last = -1;
  for (int r = lo; r < hi; ++r)
    if (row_active[r] && starts(r)) last = r;
  s_last[tid] = last;
  __syncthreads();
  for (int off = 1; off < 1024; off <<= 1) {               // inclusive maximum over the threads before and at this one
    const int v = tid >= off ? s_last[tid - off] : -1;
    __syncthreads();
    s_last[tid] = max(s_last[tid], v);
    __syncthreads();
  }
  int cur = tid > 0 ? s_last[tid - 1] : -1;                // start of the segment that reaches into this thread's rows
  const int cur0 = cur;
  for (int r = lo; r < hi; ++r) {
    if (!row_active[r]) { row_seg[r] = -1; row_j[r] = 0; continue; }
    if (starts(r)) {
      cur = r;
      const int s = atomicAdd(&s_cnt, 1);
      row_seg[r] = s;
    }
    row_j[r] = r - cur;
  }
  __syncthreads();
  cur = cur0;
  for (int r = lo; r < hi; ++r) {                          // the last row of a segment writes its descriptor
    if (!row_active[r]) continue;
    if (row_j[r] == 0) cur = r;
    const bool ends = r == R - 1 || !row_active[r + 1] || row_j[r + 1] == 0;
    if (!ends) continue;
    const int s = row_seg[cur], g = row_slot[r], start = row_pos[cur], n = r - cur + 1;
    bool ok = true;
    int par = 0;
    if (recurrent) {
      ok = atomicAdd(&claim[g], 1) == 0 && (start == 0 || start == state_len[g]);
      if (ok) { par = parity[g]; parity[g] = par ^ 1; state_len[g] = start + n; }
      else atomicAdd(err, 1);
    }
    int32_t* d = seg + (size_t)s * 8;
    d[0] = cur; d[1] = ok ? n : 0; d[2] = g; d[3] = start; d[4] = par;
    if (recurrent && ok) {
      const int nc = (n + SEG_CHUNK - 1) / SEG_CHUNK, base = atomicAdd(&s_chunks, nc);
      d[5] = base;
      for (int i = 0; i < nc; ++i) chunk[base + i] = make_int4(cur + i * SEG_CHUNK, min(SEG_CHUNK, n - i * SEG_CHUNK), s, i);
    }
  }
  __syncthreads();
  cur = cur0;
  for (int r = lo; r < hi; ++r) {
    if (!row_active[r]) continue;
    if (row_j[r] == 0) cur = r;
    const int s = row_seg[cur];
    const bool ok = seg[(size_t)s * 8 + 1] > 0;
    if (r != cur) row_seg[r] = s;
    if (!ok) row_seg[r] = -1;
  }
  __syncthreads();
  for (int r = lo; r < hi; ++r)
    if (row_seg[r] < 0) row_active[r] = 0;
  if (tid == 0) { nseg_out[0] = s_cnt; nseg_out[1] = s_chunks; }
}

// state of group src -> group dst (both tail buffers, the recurrent matrices, the length).  grid (chunks), block 256; n0, n1: floats per group
static __global__ __launch_bounds__(256) void k_state_copy(float* const* bases, const int64_t* per_group, int nbuf, int src, int dst, int32_t* state_len, int32_t* parity) {
  for (int b = 0; b < nbuf; ++b) {
    float* p = bases[b];
    const int64_t n = per_group[b];
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) p[dst * n + i] = p[src * n + i];
  }
  if (blockIdx.x == 0 && threadIdx.x == 0) { state_len[dst] = state_len[src]; parity[dst] = parity[src]; }
}
static __global__ __launch_bounds__(256) void k_latent_pages_copy(PageStateDev s, int src, int dst, char* const* pools, const int64_t* page_bytes, int P) {
  const int i = blockIdx.x, l = blockIdx.y;
  if (i >= s.num_pages_used[dst] || i >= s.num_pages_used[src]) return;
  const int64_t n = page_bytes[l];
  const u32x4* a = reinterpret_cast<const u32x4*>(pools[l] + (size_t)s.page_map[(size_t)src * s.mpg + i] * n);
  u32x4* b = reinterpret_cast<u32x4*>(pools[l] + (size_t)s.page_map[(size_t)dst * s.mpg + i] * n);
  for (int64_t e = threadIdx.x; e < n / 16; e += 256) b[e] = a[e];
}

// ---------------------------------------------------------------------------------------------------- embedding, norms
// A norm's parameters (zeros behind feature E - 1); w null: no norm.  KIND IXT_NORM_RMS: t / sqrt(mean(t^2) + eps) (1 + w); IXT_NORM_TANH: feature by
// feature tanh(alpha t) w + b; IXT_NORM_LAYER: (t - mean) / sqrt(mean((t - mean)^2) + eps) w + b; IXT_NORM_ONE: t / sqrt(mean(t^2) + eps) w[0].
struct NormW { const float *w, *b, *alpha; };
__device__ __forceinline__ void load8(const float* __restrict__ p, float* o) {       // p % 16 bytes == 0
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w; o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
}
__device__ __forceinline__ void load8(const bf16_t* __restrict__ p, float* o) {
  const u32x4 a = *reinterpret_cast<const u32x4*>(p);
  o[0] = bflo(a.x); o[1] = bfhi(a.x); o[2] = bflo(a.y); o[3] = bfhi(a.y); o[4] = bflo(a.z); o[5] = bfhi(a.z); o[6] = bflo(a.w); o[7] = bfhi(a.w);
}
__device__ __forceinline__ void store4(bf16_t* p, const float* v) {
  uint2 o;
  o.x = pack2(f2bf(v[0]), f2bf(v[1])); o.y = pack2(f2bf(v[2]), f2bf(v[3]));
  *reinterpret_cast<uint2*>(p) = o;
}
__device__ __forceinline__ void store4(float* p, const float* v) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
// What a norm needs to know of a row: s = the tanh norm's alpha, or 1 / sqrt(mean + eps); mu: the layer norm's mean.
struct NormStat { float s, mu; };
// 8 features k0 .. k0 + 7 through a norm
template <int KIND>
__device__ __forceinline__ void norm8(const NormW& n, NormStat st, int k0, const float* t, float* o) {
  const float s = st.s;
  float w[8], b[8];
  if constexpr (KIND == IXT_NORM_ONE) {
    const float g = s * n.w[0];
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = t[j] * g;
    return;
  }
  load8(n.w + k0, w);
  if constexpr (KIND == IXT_NORM_TANH) {
    load8(n.b + k0, b);
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = fmaf(tanh_f32(s * t[j]), w[j], b[j]);
  } else if constexpr (KIND == IXT_NORM_LAYER) {
    load8(n.b + k0, b);
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = fmaf((t[j] - st.mu) * s, w[j], b[j]);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = t[j] * s * (1.0f + w[j]);
  }
}

// Statistics of a row that a block of 256 holds as v[NI][8] (features i 2048 + 8 tid + j, zeros behind feature E - 1)
template <int KIND, int NI>
__device__ __forceinline__ NormStat row_stat(const NormW& n, const float (*v)[8], int E, float eps, float* red) {
  if constexpr (KIND == IXT_NORM_TANH) return NormStat{*n.alpha, 0.0f};
  float mu = 0.0f, ss = 0.0f;
  if constexpr (KIND == IXT_NORM_LAYER) {
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int j = 0; j < 8; ++j) mu += v[i][j];
    mu = block_sum256(mu, red) / (float)E;
  }
#pragma unroll
  for (int i = 0; i < NI; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (i * 2048 + (int)threadIdx.x * 8 + j < E) ss = fmaf(v[i][j] - mu, v[i][j] - mu, ss);
  return NormStat{1.0f / sqrtf(block_sum256(ss, red) / (float)E + eps), mu};
}
// Hyper-connections.  A sublayer's numbers: HC_IN, HC_OUT [HC_MAX] each, then mix [from][to], rows HC_MAX apart.
#define HC_MAX 16
struct HyperW { const float *in, *out, *mix; };      // in: of the sublayer that follows (nullptr: none does); out, mix: of the one that ends

// x[r] = table[token] * scale (f32; `streams` copies of it) and its copy as the first dot's operand, through a tanh norm if `pre` is one.  cat (nullptr: none):
// act of two Ep columns, the row as it is in both halves.  grid R, block 256.
template <typename T>
__global__ __launch_bounds__(256) void k_embed_scaled(const T* __restrict__ table, const int32_t* __restrict__ ids, float scale, int E, int Ep, int V, int streams, NormW pre,
                                                      float* __restrict__ x, T* __restrict__ xb, T* __restrict__ cat) {
  x += (size_t)blockIdx.x * (streams - 1) * E;             // rows are `streams` E apart
  const int r = blockIdx.x;
  const int id = min(max(ids[r], 0), V - 1);
  for (int k0 = threadIdx.x * 8; k0 < Ep; k0 += 2048) {
    float v[8];
    if ((E & 7) == 0 && k0 < E) {
      load8(table + (size_t)id * E + k0, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] *= scale;
      for (int s = 0; s < streams; ++s) { store4(x + (size_t)(r + s) * E + k0, v); store4(x + (size_t)(r + s) * E + k0 + 4, v + 4); }
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        v[j] = k0 + j < E ? to_f(table[(size_t)id * E + k0 + j]) * scale : 0.0f;
        if (k0 + j < E)
          for (int s = 0; s < streams; ++s) x[(size_t)(r + s) * E + k0 + j] = v[j];
      }
    }
    if (cat != nullptr) { act_store8(cat, r, k0, 2 * Ep, v); act_store8(cat, r, Ep + k0, 2 * Ep, v); }
    if (pre.w != nullptr) norm8<IXT_NORM_TANH>(pre, NormStat{*pre.alpha, 0.0f}, k0, v, v);
    act_store8(xb, r, k0, Ep, v);
  }
}

// A sublayer's output t (slices, or the weighted sum of a row's expert outputs) -> norm behind the sublayer -> residual -> norm in front of the next one:
//   x <- x + post(t);  xb = pre(x) as the next dot's operand, h32 (if given) the same in f32.
// t.n == 0: t = 0 and x stays.  pos != nullptr: t = sum_j wts[r][j] * slices row pos[r][j].  add.n > 0: its row, times addw[r] if that is given, joins t.
// bias, times fbias, joins t; fresh != 0: t takes the place of x instead of joining it.
// shift.mu != nullptr (every row the only one of its page group): the operand is h + (h' - h) mu of h = pre(x), h' the group's h of one token before.
// SM > 0: `streams` (<= SM) streams in the place of x ([R][streams][E]): x_t <- sum_s mix[s][t] x_s + out[t] post(t), and pre takes sum_s in[s] x_s.
// A thread owns 8 consecutive features of every 2048 (NI times).  grid R, block 256.
// Token shift: mu (zeros behind feature E - 1); the group's last h [group][2][Ep], read at one parity and written at the other (k_segments)
struct ShiftArgs { const float* mu; float* state; const int32_t *slot, *pos, *active, *parity; };
struct SubNormArgs {
  Slices t, add; const float* addw;
  const int32_t* pos; const float* wts; int top;
  NormW post, pre; float eps; int E, Ep, streams; HyperW hc;
  const float* bias; float fbias; int fresh; ShiftArgs shift; int Kp;      // Kp: columns of the operand's rows
};
template <typename T, int NI, int KIND, int SM>
__global__ __launch_bounds__(256) void k_sub_norm(SubNormArgs a, float* __restrict__ x, T* __restrict__ xb, float* __restrict__ h32) {
  __shared__ float red[4];
  const Slices &t = a.t, &add = a.add;
  const int32_t* __restrict__ pos = a.pos;
  const float* __restrict__ wts = a.wts;
  const NormW &post = a.post, &pre = a.pre;
  const int r = blockIdx.x, top = a.top, E = a.E, Ep = a.Ep;
  const bool vec = (E & 3) == 0;
  float v[NI][8], xv[NI][8];
  constexpr bool AHEAD = NI <= 2 && SM == 0;               // the group's last h is requested before anything else
  [[maybe_unused]] float old[AHEAD ? NI : 1][8];
  const float* before = nullptr;                           // the group's last h, and where this one goes
  float* keep = nullptr;
  if (SM == 0 && a.shift.mu != nullptr) {
    const int active = a.shift.active[r], grp = a.shift.slot[r], pos = a.shift.pos[r];
    if (active) {
      const int par = a.shift.parity[grp] ^ 1;
      float* base = a.shift.state + (size_t)grp * 2 * Ep;
      if (pos > 0) before = base + (size_t)par * Ep;
      keep = base + (size_t)(par ^ 1) * Ep;
    }
    if constexpr (AHEAD) {
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int k0 = i * 2048 + threadIdx.x * 8;
#pragma unroll
        for (int j = 0; j < 8; ++j) old[i][j] = 0.0f;
        if (before != nullptr && k0 < Ep) load8(before + k0, old[i]);
      }
    }
  }
  constexpr bool EARLY = SM > 0 && NI * SM <= 8;           // the streams are requested before anything else
  float4 es[EARLY ? NI * SM * 2 : 1];
  if constexpr (EARLY) {
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
      for (int s = 0; s < SM; ++s)
#pragma unroll
        for (int q = 0; q < 2; ++q) {
          const int k = i * 2048 + threadIdx.x * 8 + q * 4;
          if (vec && k < E && s < a.streams) es[(i * SM + s) * 2 + q] = *reinterpret_cast<const float4*>(x + ((size_t)r * a.streams + s) * E + k);
        }
  }
  const float fadd = a.addw != nullptr ? a.addw[r] : 1.0f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int k0 = i * 2048 + threadIdx.x * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j) v[i][j] = xv[i][j] = 0.0f;
#pragma unroll
    for (int q = 0; q < 8; q += 4) {
      if (k0 + q >= E) continue;
      if (pos == nullptr) {
        if (t.n > 0) t.template at4<NI == 1 ? 10 : 4>(r, k0 + q, v[i] + q);
      } else {
        for (int j = 0; j < top; ++j) {
          float u[4];
          t.at4(pos[(size_t)r * top + j], k0 + q, u);
          const float wj = wts[(size_t)r * top + j];
#pragma unroll
          for (int e = 0; e < 4; ++e) v[i][q + e] = fmaf(wj, u[e], v[i][q + e]);
        }
      }
      if (add.n > 0) {
        float u[4];
        add.at4(r, k0 + q, u);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[i][q + e] = fmaf(fadd, u[e], v[i][q + e]);
      }
      if (a.bias != nullptr) {
        const float4 b = *reinterpret_cast<const float4*>(a.bias + k0 + q);
        v[i][q] = fmaf(a.fbias, b.x, v[i][q]); v[i][q + 1] = fmaf(a.fbias, b.y, v[i][q + 1]); v[i][q + 2] = fmaf(a.fbias, b.z, v[i][q + 2]); v[i][q + 3] = fmaf(a.fbias, b.w, v[i][q + 3]);
      }
      if (SM > 0 || a.fresh) continue;
      if (vec) {
        const float4 xx = *reinterpret_cast<const float4*>(x + (size_t)r * E + k0 + q);
        xv[i][q] = xx.x; xv[i][q + 1] = xx.y; xv[i][q + 2] = xx.z; xv[i][q + 3] = xx.w;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (k0 + q + e < E) xv[i][q + e] = x[(size_t)r * E + k0 + q + e];
      }
    }
  }
  if (t.n > 0 && post.w != nullptr) {
    const NormStat st = row_stat<KIND, NI>(post, v, E, a.eps, red);
#pragma unroll
    for (int i = 0; i < NI; ++i)
      if (i * 2048 + (int)threadIdx.x * 8 < Ep) norm8<KIND>(post, st, i * 2048 + threadIdx.x * 8, v[i], v[i]);
  }
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int k0 = i * 2048 + threadIdx.x * 8;
    if (k0 >= Ep) continue;
    if constexpr (SM > 0) {                                  // (features behind E - 1 are never read; xv stays 0 there)
      float* xr = x + (size_t)r * a.streams * E;
#pragma unroll
      for (int q = 0; q < 8; q += 4) {
        if (k0 + q >= E) continue;
        float old[SM][4];
#pragma unroll
        for (int s = 0; s < SM; ++s) {
          old[s][0] = old[s][1] = old[s][2] = old[s][3] = 0.0f;
          if (s >= a.streams) continue;
          const float* p = xr + (size_t)s * E + k0 + q;
          if (vec) { const float4 u = EARLY ? es[EARLY ? (i * SM + s) * 2 + q / 4 : 0] : *reinterpret_cast<const float4*>(p); old[s][0] = u.x; old[s][1] = u.y; old[s][2] = u.z; old[s][3] = u.w; }
          else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (k0 + q + e < E) old[s][e] = p[e];
          }
        }
#pragma unroll SM <= 4 ? SM : 1
        for (int d = 0; d < (SM <= 4 ? SM : a.streams); ++d) {
          if (d >= a.streams) continue;
          float nw[4];
          float* p = xr + (size_t)d * E + k0 + q;
          if (t.n > 0) {
            const float fo = a.hc.out[d];
#pragma unroll
            for (int e = 0; e < 4; ++e) nw[e] = fo * v[i][q + e];
#pragma unroll
            for (int s = 0; s < SM; ++s) {
              const float fm = a.hc.mix[s * HC_MAX + d];      // (rows behind the last stream are zero)
#pragma unroll
              for (int e = 0; e < 4; ++e) nw[e] = fmaf(fm, old[s][e], nw[e]);
            }
            if (vec) *reinterpret_cast<float4*>(p) = make_float4(nw[0], nw[1], nw[2], nw[3]);
            else {
#pragma unroll
              for (int e = 0; e < 4; ++e)
                if (k0 + q + e < E) p[e] = nw[e];
            }
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) nw[e] = k0 + q + e < E ? p[e] : 0.0f;
          }
          if (a.hc.in != nullptr) {
            const float fi = a.hc.in[d];
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (k0 + q + e < E) xv[i][q + e] = fmaf(fi, nw[e], xv[i][q + e]);
          }
        }
      }
      continue;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) xv[i][j] = k0 + j < E ? xv[i][j] + v[i][j] : 0.0f;
    if (t.n > 0) {
      if (vec) {
#pragma unroll
        for (int q = 0; q < 8; q += 4)
          if (k0 + q < E) *reinterpret_cast<float4*>(x + (size_t)r * E + k0 + q) = make_float4(xv[i][q], xv[i][q + 1], xv[i][q + 2], xv[i][q + 3]);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (k0 + j < E) x[(size_t)r * E + k0 + j] = xv[i][j];
      }
    }
  }
  if (SM > 0 && a.hc.in == nullptr) return;                // the head takes the streams themselves
  NormStat st{};
  if (pre.w != nullptr) st = row_stat<KIND, NI>(pre, xv, E, a.eps, red);
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int k0 = i * 2048 + threadIdx.x * 8;
    if (k0 >= Ep) continue;
    if (pre.w != nullptr) norm8<KIND>(pre, st, k0, xv[i], xv[i]);      // (w and b are zero behind feature E - 1)
    if (h32 != nullptr) {
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (k0 + j < E) h32[(size_t)r * E + k0 + j] = xv[i][j];
    }
    if (SM == 0 && a.shift.mu != nullptr) {
      float mu[8], od[8] = {0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f};
      load8(a.shift.mu + k0, mu);
      if constexpr (AHEAD) {
#pragma unroll
        for (int j = 0; j < 8; ++j) od[j] = old[i][j];
      } else if (before != nullptr) load8(before + k0, od);
      if (keep != nullptr) { store4(keep + k0, xv[i]); store4(keep + k0 + 4, xv[i] + 4); }
#pragma unroll
      for (int j = 0; j < 8; ++j) xv[i][j] = fmaf(od[j] - xv[i][j], mu[j], xv[i][j]);
    }
    if (xb != nullptr) act_store8(xb, r, k0, a.Kp, xv[i]);
  }
}

// Token shift over runs of rows: the operand is h + (h' - h) mu, h' the row before, or (first of its run) what the group has kept; the run's last row leaves
// its own.  h [R][E], state as in ShiftArgs.  grid R, block 256.
template <typename T>
__global__ __launch_bounds__(256) void k_token_shift(const float* __restrict__ h, const float* __restrict__ mu, float* __restrict__ state, const int32_t* __restrict__ row_seg,
                                                     const int32_t* __restrict__ row_j, const int32_t* __restrict__ seg, int E, int Ep, T* __restrict__ xb) {
  const int r = blockIdx.x, s = row_seg[r], j = row_j[r];
  if (s < 0) return;
  const int32_t* sg = seg + (size_t)s * 8;
  const int n = sg[1], start = sg[3], par = sg[4];
  float* base = state + (size_t)sg[2] * 2 * Ep;
  const float *hr = h + (size_t)r * E, *before = j > 0 ? hr - E : start > 0 ? base + (size_t)par * Ep : nullptr;
  float* keep = j == n - 1 ? base + (size_t)(par ^ 1) * Ep : nullptr;
  for (int k0 = threadIdx.x * 8; k0 < Ep; k0 += 2048) {
    float v[8], old[8], m[8];
    load8(mu + k0, m);
    if ((E & 3) == 0 && k0 + 8 <= E) {
      load8(hr + k0, v);
      if (before != nullptr) load8(before + k0, old);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        v[i] = k0 + i < E ? hr[k0 + i] : 0.0f;
        if (before != nullptr) old[i] = k0 + i < E ? before[k0 + i] : 0.0f;
      }
    }
    if (keep != nullptr) { store4(keep + k0, v); store4(keep + k0 + 4, v + 4); }
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = fmaf((before != nullptr ? old[i] : 0.0f) - v[i], m[i], v[i]);
    act_store8(xb, r, k0, Ep, v);
  }
}

// rows lrows[i] (or lrow0 + i) of x (the sum of their streams) -> the model's norm -> the head's operand.  grid nl, block 256.
template <typename T, int NI, int KIND>
__global__ __launch_bounds__(256) void k_final_norm(const float* __restrict__ x, const int32_t* __restrict__ lrows, int lrow0, int nrows, int streams, NormW w, float eps, int E,
                                                    int Ep, T* __restrict__ xn) {
  __shared__ float red[4];
  const int r = min(max(lrows != nullptr ? lrows[blockIdx.x] : lrow0 + (int)blockIdx.x, 0), nrows - 1);
  float v[NI][8];
#pragma unroll
  for (int i = 0; i < NI; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int k = i * 2048 + threadIdx.x * 8 + j;
      v[i][j] = 0.0f;
      if (k < E)
        for (int s = 0; s < streams; ++s) v[i][j] += x[((size_t)r * streams + s) * E + k];
    }
  const NormStat st = row_stat<KIND, NI>(w, v, E, eps, red);
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int k0 = i * 2048 + threadIdx.x * 8;
    if (k0 >= Ep) continue;
    norm8<KIND>(w, st, k0, v[i], v[i]);
    act_store8(xn, blockIdx.x, k0, Ep, v[i]);
  }
}
// the residual stream as one row per token: the sum of its streams.  grid (R, ceil(E / 256)), block 256.
static __global__ __launch_bounds__(256) void k_stream_sum(const float* __restrict__ x, int streams, int E, float* __restrict__ out) {
  const int r = blockIdx.x, k = blockIdx.y * 256 + threadIdx.x;
  if (k >= E) return;
  float v = 0.0f;
  for (int s = 0; s < streams; ++s) v += x[((size_t)r * streams + s) * E + k];
  out[(size_t)r * E + k] = v;
}

// logits = the head's slices times scale; (max, first index) per block of 1024 columns over the allowed ones.  grid (ceil(V / 1024), nl), block 256.
static __global__ __launch_bounds__(256) void k_head_post(Slices t, int V, float scale, ColRanges cr, float* __restrict__ logits /*[nl][V] or nullptr*/, float* __restrict__ amax_val,
                                                   int32_t* __restrict__ amax_idx) {
  __shared__ float bv[4];
  __shared__ int bi[4];
  const int r = blockIdx.y, lane = threadIdx.x & 63;
  float best = -INFINITY;
  int idx = 0x7fffffff;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = blockIdx.x * 1024 + i * 256 + threadIdx.x;
    if (c >= V) continue;
    const float v = t.at(r, c) * scale;
    if (logits != nullptr) logits[(size_t)r * V + c] = v;
    if (v > best && col_allowed(cr, c)) { best = v; idx = c; }
  }
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const float ov = __shfl_xor(best, off, 64);
    const int oi = __shfl_xor(idx, off, 64);
    if (ov > best || (ov == best && oi < idx)) { best = ov; idx = oi; }
  }
  if (lane == 0) { bv[threadIdx.x >> 6] = best; bi[threadIdx.x >> 6] = idx; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 4; ++w)
      if (bv[w] > best || (bv[w] == best && bi[w] < idx)) { best = bv[w]; idx = bi[w]; }
    amax_val[(size_t)r * gridDim.x + blockIdx.x] = best;
    amax_idx[(size_t)r * gridDim.x + blockIdx.x] = idx;
  }
}

// ---------------------------------------------------------------------------------------------------- tiles of cached rows
// Tiles of 64 cached rows of D elements (D a multiple of 32) in LDS, for the matrix cores.  Groups of 8 pieces of 16 bytes (64 features), each [64 rows]
// [8 pieces]; piece c of row r lies at place c ^ (r & 7), so that neither the score operand (16 rows x 16 bytes) nor the column-wise reads of the value
// operand (ds_read_b64_tr_b16: 4 rows x 16 columns) pile up on a bank.  D an odd multiple of 32: a last group of 4 pieces, [64 rows][4 pieces], place
// c ^ (r & 3).  A wave load (1 KiB) is 8 rows of a group (16 of the last), so all its addresses are two (three) row pointers plus constants.
// 64 cached rows -> LDS: `off` = the row that this lane's key (key lane of the tile) occupies in the pool
template <int D>
__device__ __forceinline__ void tile_dma(const bf16_t* __restrict__ pages, int off, bf16_t* tile, int wave, int lane) {
  constexpr int NG = D / 64;
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int o = __shfl(off, (wave + 4 * j) * 8 + (lane >> 3), 64);
    const bf16_t* src = pages + (size_t)o * D + ((lane & 7) ^ (lane >> 3)) * 8;
#pragma unroll
    for (int gr = 0; gr < NG; ++gr)
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(src + gr * 64),
                                       (__attribute__((address_space(3))) void*)(tile + gr * 4096 + (wave + 4 * j) * 512), 16, 0, 0);
  }
  if constexpr (D % 64 != 0) {
    const int o = __shfl(off, wave * 16 + (lane >> 2), 64);
    const bf16_t* src = pages + (size_t)o * D + NG * 64 + ((lane & 3) ^ ((lane >> 2) & 3)) * 8;
    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src, (__attribute__((address_space(3))) void*)(tile + NG * 4096 + wave * 512), 16, 0, 0);
  }
}
// piece c (features 8 c .. 8 c + 7) of row r of a tile
template <int D>
__device__ __forceinline__ void tile_put(bf16_t* tile, int r, int c, u32x4 v) {
  bf16_t* p = c < D / 64 * 8 ? tile + (c >> 3) * 4096 + r * 64 + ((c ^ r) & 7) * 8 : tile + D / 64 * 4096 + r * 32 + ((c ^ r) & 3) * 8;
  *reinterpret_cast<u32x4*>(p) = v;
}
__device__ __forceinline__ int cached_row(const int32_t* __restrict__ prow, int key, int pshift) { return (prow[key >> pshift] << pshift) + (key & ((1 << pshift) - 1)); }
// where a lane reads in a tile (byte offsets; the rest of every address is a constant)
struct TileLane {
  uint32_t k0, k1, kh;      // score operand: row r_in, even / odd steps of a full group, the half group
  uint32_t v[4];            // value operand: row 4 q + a, column tiles 0 .. 3 of a group (lane 4 a + p of a 16-lane group: columns 4 p .. 4 p + 3)
  uint32_t vh[2];           // the same, column tiles 0 and 1 of the half group
};
__device__ __forceinline__ TileLane tile_lane(int r_in, int cq) {
  TileLane L;
  L.k0 = r_in * 128 + ((cq ^ (r_in & 7)) * 16);
  L.k1 = r_in * 128 + (((4 + cq) ^ (r_in & 7)) * 16);
  L.kh = r_in * 64 + ((cq ^ (r_in & 3)) * 16);
  const int row = 4 * cq + (r_in >> 2), p = r_in & 3;
#pragma unroll
  for (int i = 0; i < 4; ++i) L.v[i] = row * 128 + (((2 * i + (p >> 1)) ^ (row & 7)) * 16) + (p & 1) * 8;
#pragma unroll
  for (int i = 0; i < 2; ++i) L.vh[i] = row * 64 + (((2 * i + (p >> 1)) ^ (row & 3)) * 16) + (p & 1) * 8;
  return L;
}
// score operand of step ks, rows 16 n .. 16 n + 15
template <int D>
__device__ __forceinline__ bf16x8 tile_kf(const char* tile, const TileLane& L, int ks, int n) {
  if (D % 64 != 0 && ks == D / 64 * 2) return __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(tile + L.kh + D / 64 * 8192 + n * 1024));
  return __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(tile + ((ks & 1) ? L.k1 : L.k0) + (ks >> 1) * 8192 + n * 2048));
}
// value operand of column tiles 4 G .. 4 G + 3 (group G), keys 32 U + 4 q .. + 3 and 32 U + 16 + 4 q .. + 3 for lane group q; tb = LDS address of the tile
#define IXT_TILE_VT(F_, TB_, L_, G_, U_)                                                                                                                    \
  do {                                                                                                                                                        \
    _Pragma("unroll") for (int i_ = 0; i_ < 4; ++i_) {                                                                                                        \
      asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(F_[i_][0]) : "v"((TB_) + (L_).v[i_]), "n"((G_) * 8192 + (U_) * 4096) : "memory");              \
      asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(F_[i_][1]) : "v"((TB_) + (L_).v[i_]), "n"((G_) * 8192 + (U_) * 4096 + 2048) : "memory");       \
    }                                                                                                                                                         \
  } while (0)
// the two column tiles of the half group G
#define IXT_TILE_VTH(F_, TB_, L_, G_, U_)                                                                                                                     \
  do {                                                                                                                                                        \
    _Pragma("unroll") for (int i_ = 0; i_ < 2; ++i_) {                                                                                                        \
      asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(F_[i_][0]) : "v"((TB_) + (L_).vh[i_]), "n"((G_) * 8192 + (U_) * 2048) : "memory");             \
      asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(F_[i_][1]) : "v"((TB_) + (L_).vh[i_]), "n"((G_) * 8192 + (U_) * 2048 + 1024) : "memory");      \
    }                                                                                                                                                         \
  } while (0)
// all but the youngest N_ reads have been delivered: everything that uses the NF_ operands F_ comes behind this
#define IXT_TILE_VWAITN(F_, NF_, N_)                                                                                                                          \
  do {                                                                                                                                                        \
    asm volatile("s_waitcnt lgkmcnt(%0)" ::"n"(N_) : "memory");                                                                                               \
    __builtin_amdgcn_sched_barrier(0);                                                                                                                        \
    _Pragma("unroll") for (int i_ = 0; i_ < (NF_); ++i_) asm volatile("" : "+v"(F_[i_][0]), "+v"(F_[i_][1]));                                                  \
  } while (0)
#define IXT_TILE_VWAIT(F_, N_) IXT_TILE_VWAITN(F_, 4, N_)
__device__ __forceinline__ uint32_t lds_addr(const void* p) { return (uint32_t)(uintptr_t)((const __attribute__((address_space(3))) void*)(p)); }
__device__ __forceinline__ bf16x8 tile_vfrag(const uint2 (&f)[2]) {
  u32x4 v; v.x = f[0].x; v.y = f[0].y; v.z = f[1].x; v.w = f[1].y;
  return __builtin_bit_cast(bf16x8, v);
}

// ---------------------------------------------------------------------------------------------------- latent attention
struct LatentGeom {
  int H, dn, dr, rank, P, mpg, window;      // heads, unrotated / rotated query dims, latent size, page size, pages per group, window (<= 0: none)
  int rankp, rotp;                          // padded sizes: cached row = [rankp latent | rotp rotated key part], DK = rankp + rotp elements
  float scale;
};

// The input projection's slices t (d_off: latent, rotated key part) -> the row's cache entry (normed latent, rotated key part); the queries' slices tq
// (heads of dn + dr, columns from 0 on) -> unrotated parts head-major as the operand of the key up-projection (row h Rp + r), rotated parts qr
// [R][H][rotp].  rope: f32 [position][dr / 2] cos, sin.  grid (R, 1 + ceil(H / 4)), block 256: y = 0 the cache entry, y > 0 four heads (a wave each).
template <typename T>
__global__ __launch_bounds__(256) void k_latent_prep(Slices t, Slices tq, int d_off, LatentGeom g, const float* __restrict__ cnorm, float eps, const float* __restrict__ rope_cos,
                                                     const float* __restrict__ rope_sin, const int32_t* __restrict__ row_slot, const int32_t* __restrict__ row_pos,
                                                     const int32_t* __restrict__ row_active, const int32_t* __restrict__ page_map, T* __restrict__ pages, T* __restrict__ qx,
                                                     int dnp, int Rp, T* __restrict__ qr) {
  __shared__ float red[4];
  const int r = blockIdx.x, half = g.dr >> 1;
  const bool act = row_active[r] != 0;
  const int pos = act ? row_pos[r] : 0;
  if (blockIdx.y == 0) {
    if (!act) return;
    float ss = 0.0f;
    for (int k = threadIdx.x; k < g.rank; k += 256) { const float v = t.at(r, d_off + k); ss = fmaf(v, v, ss); }
    const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)g.rank + eps);
    const int page = page_map[(size_t)row_slot[r] * g.mpg + pos / g.P];
    T* row = pages + ((size_t)page * g.P + pos % g.P) * (g.rankp + g.rotp);
    for (int k = threadIdx.x; k < g.rank; k += 256) row[k] = from_f<T>(t.at(r, d_off + k) * rs * cnorm[k]);
    for (int i = threadIdx.x; i < half; i += 256) {
      const float u = t.at(r, d_off + g.rank + 2 * i), v = t.at(r, d_off + g.rank + 2 * i + 1);
      const float c = rope_cos[(size_t)pos * half + i], s = rope_sin[(size_t)pos * half + i];
      row[g.rankp + 2 * i] = from_f<T>(u * c - v * s);
      row[g.rankp + 2 * i + 1] = from_f<T>(v * c + u * s);
    }
    return;
  }
  const int h = (blockIdx.y - 1) * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (h >= g.H) return;
  const int c0 = h * (g.dn + g.dr);
  for (int k = lane; k < dnp; k += 64) act_store1(qx, h * Rp + r, k, dnp, k < g.dn ? tq.at(r, c0 + k) : 0.0f);
  T* qo = qr + ((size_t)r * g.H + h) * g.rotp;
  for (int i = lane; i < g.rotp / 2; i += 64) {
    float a = 0.0f, b = 0.0f;
    if (i < half) {
      const float u = tq.at(r, c0 + g.dn + 2 * i), v = tq.at(r, c0 + g.dn + 2 * i + 1);
      const float c = rope_cos[(size_t)pos * half + i], s = rope_sin[(size_t)pos * half + i];
      a = u * c - v * s; b = v * c + u * s;
    }
    qo[2 * i] = from_f<T>(a); qo[2 * i + 1] = from_f<T>(b);
  }
}

// n columns of a projection from c0 on, RMS-normed with a plain weight, as the next dot's operand.  grid R, block 256.
template <typename T>
__global__ __launch_bounds__(256) void k_rms_x(Slices t, int c0, int n, const float* __restrict__ w, float eps, T* __restrict__ out, int Kp) {
  __shared__ float red[4];
  const int r = blockIdx.x;
  float ss = 0.0f;
  for (int k = threadIdx.x; k < n; k += 256) { const float v = t.at(r, c0 + k); ss = fmaf(v, v, ss); }
  const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)n + eps);
  for (int k = threadIdx.x; k < Kp; k += 256) act_store1(out, r, k, Kp, k < n ? t.at(r, c0 + k) * rs * w[k] : 0.0f);
}

// Any sizes (rank <= 1024), any T: block = (row, head); thread = key for the scores (tiles of 256 keys, running maximum and sum), thread = latent
// column for the weighted sum.  qa: slices of the queries in latent space (row h Rp + r); out: act(T), row h Rp + r.  grid (R, H), block 256,
// LDS = (rankp + rotp + 256) floats.
template <typename T>
__global__ __launch_bounds__(256) void k_latent_attn_any(Slices qa, const T* __restrict__ qr, LatentGeom g, const int32_t* __restrict__ row_slot, const int32_t* __restrict__ row_pos,
                                                         const int32_t* __restrict__ row_active, const int32_t* __restrict__ page_map, const T* __restrict__ pages, int Rp,
                                                         T* __restrict__ out, int Kp) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[4];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, DK = g.rankp + g.rotp;
  if (!row_active[r]) return;
  float* q = sm;
  float* p = sm + DK;
  for (int k = tid; k < DK; k += 256) {
    float v = 0.0f;
    if (k < g.rank) v = qa.at(h * Rp + r, k);
    else if (k >= g.rankp) v = to_f(qr[((size_t)r * g.H + h) * g.rotp + k - g.rankp]);
    q[k] = to_f(from_f<T>(v));
  }
  __syncthreads();
  const int pos = row_pos[r], k_lo = g.window > 0 ? max(0, pos - g.window + 1) : 0;
  const int32_t* prow = page_map + (size_t)row_slot[r] * g.mpg;
  float m = -INFINITY, l = 0.0f, acc[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int j0 = k_lo; j0 <= pos; j0 += 256) {
    const int j = j0 + tid;
    float s = -INFINITY;
    if (j <= pos) {
      const T* kp = pages + ((size_t)prow[j / g.P] * g.P + j % g.P) * DK;
      float a = 0.0f;
      for (int k = 0; k < g.rank; ++k) a = fmaf(q[k], to_f(kp[k]), a);
      float b = 0.0f;
      for (int k = g.rankp; k < g.rankp + g.dr; ++k) b = fmaf(q[k], to_f(kp[k]), b);
      s = (a + b) * g.scale;
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
      const T* kp = pages + ((size_t)prow[(j0 + kk) / g.P] * g.P + (j0 + kk) % g.P) * DK;
      const float w = p[kk];
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (tid + 256 * i < g.rank) acc[i] = fmaf(w, to_f(kp[tid + 256 * i]), acc[i]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (tid + 256 * i < Kp) act_store1(out, h * Rp + r, tid + 256 * i, Kp, tid + 256 * i < g.rank ? acc[i] / l : 0.0f);
}

// The bf16 matrix-core forms.  All heads of a row share the cached latent, so the M side of the products is (row, head) pairs and every cached row is
// read once for all of them.  Keys come in tiles of 64 by LDS-DMA (no registers in between).
//   scores   D[key][pair] = mfma(A = cached rows, B = queries [latent | rotated]): a lane holds 4 keys of one pair per product
//   weights  running maximum / sum per pair in f32, exp2; P goes to bf16
//   output   D[column][pair] = mfma(A = cached latent read column-wise, B = P)
// RT = 16-column tiles of the padded latent, RS = 32-wide steps of the padded rotated part.
struct LatentAttnArgs {
  Slices qa; const bf16_t* qr; LatentGeom g;
  const int32_t *row_slot, *row_pos, *row_active, *page_map;
  const bf16_t* pages;
  int R, Rp, NQ, HB, pshift;
  bf16_t* out; int Kp;                     // act, row h Rp + r
  float *part_o, *part_ml;                 // splits > 1: [R H][splits][rankp], [R H][splits][2]
};
template <int RT, int RS> struct LatentTile {
  static_assert(RT % 4 == 0 && (RS == 1 || RS == 2), "whole groups of the latent; one group or half a group of the rotated part");
  static constexpr int DK = RT * 16 + RS * 32, NKS = RT / 2 + RS;                               // elements per row, score steps
  static constexpr int BYTES = 64 * DK * 2;
};
__device__ __forceinline__ bf16x8 latent_q8(const LatentAttnArgs& a, int qrow, int c) {
  float v[8];
  a.qa.at4(qrow, c, v);
  a.qa.at4(qrow, c + 4, v + 4);
  u32x4 o;
  o.x = pack2(f2bf(v[0]), f2bf(v[1])); o.y = pack2(f2bf(v[2]), f2bf(v[3])); o.z = pack2(f2bf(v[4]), f2bf(v[5])); o.w = pack2(f2bf(v[6]), f2bf(v[7]));
  return __builtin_bit_cast(bf16x8, o);
}
// Prompts: a block owns 64 pairs = up to 64 / HB consecutive rows x HB heads (a wave 16 of them), all waves walk the same key tiles, the next tile
// arriving while the current one is used.  P stays in registers: with the key order 4q .. 4q + 3, 16 + 4q .. 16 + 4q + 3 per lane group q of 32
// keys, the lane's own scores ARE its operand of the next product.  grid (ceil(R / NQ), ceil(H / HB)), block 256, LDS two tiles.
template <int RT, int RS>
__global__ __launch_bounds__(256, 1) void k_latent_attn(LatentAttnArgs a) {
  typedef LatentTile<RT, RS> T;
  extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
  const LatentGeom& g = a.g;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r_in = lane & 15, cq = lane >> 4;
  const int r0 = blockIdx.x * a.NQ, nr = min(a.NQ, a.R - r0), h0 = blockIdx.y * a.HB, hb = min(a.HB, g.H - h0);
  const int pair = wave * 16 + r_in, qi = pair / a.HB, hh = pair % a.HB;
  const bool pair_ok = qi < nr && hh < hb;
  const int row = r0 + (pair_ok ? qi : 0), head = h0 + (pair_ok ? hh : 0);
  const bool live = pair_ok && a.row_active[row] != 0;
  const int pos = live ? a.row_pos[row] : -1;
  bf16x8 qf[T::NKS];                                      // queries: lane = pair r_in, 8 consecutive features per step
#pragma unroll
  for (int ks = 0; ks < RT / 2; ++ks) qf[ks] = latent_q8(a, head * a.Rp + row, ks * 32 + cq * 8);
#pragma unroll
  for (int ks = 0; ks < RS; ++ks)
    qf[RT / 2 + ks] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(a.qr + ((size_t)row * g.H + head) * g.rotp + ks * 32 + cq * 8));
  f32x4 o[RT];
#pragma unroll
  for (int i = 0; i < RT; ++i) o[i] = f32x4(0.0f);
  float m = -INFINITY, l = 0.0f;
  const float sc = g.scale * 1.44269504088896340736f;
  const TileLane L = tile_lane(r_in, cq);
  for (int ra = 0; ra < nr;) {                            // runs of rows that share a page group
    if (!a.row_active[r0 + ra]) { ++ra; continue; }
    const int slot = a.row_slot[r0 + ra];
    int lo = a.row_pos[r0 + ra], hi = lo, rb = ra + 1;
    while (rb < nr && a.row_active[r0 + rb] && a.row_slot[r0 + rb] == slot) { const int p = a.row_pos[r0 + rb]; lo = min(lo, p); hi = max(hi, p); ++rb; }
    const bool mine = live && qi >= ra && qi < rb;
    ra = rb;
    const int k_lo = g.window > 0 ? max(0, lo - g.window + 1) : 0;
    const int ntile = (hi - k_lo) / 64 + 1;
    const int32_t* prow = a.page_map + (size_t)slot * g.mpg;
    const int my_lo = g.window > 0 ? max(0, pos - g.window + 1) : 0;
    __syncthreads();                                      // the previous run's last tile has been read
    int off = cached_row(prow, min(k_lo + lane, hi), a.pshift);
    tile_dma<T::DK>(a.pages, off, lds, wave, lane);
    off = cached_row(prow, min(k_lo + 64 + lane, hi), a.pshift);
    for (int t = 0; t < ntile; ++t) {
      const bf16_t* tile = lds + (size_t)(t & 1) * 64 * T::DK;
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      __syncthreads();                                    // the tile is there; every wave is done with the other one
      if (t + 1 < ntile) {
        tile_dma<T::DK>(a.pages, off, lds + (size_t)((t + 1) & 1) * 64 * T::DK, wave, lane);
        off = cached_row(prow, min(k_lo + (t + 2) * 64 + lane, hi), a.pshift);
      }
      f32x4 s[4];
#pragma unroll
      for (int n = 0; n < 4; ++n) s[n] = f32x4(0.0f);
      bf16x8 kf[2][4];                                    // operands one step ahead of the products
#pragma unroll
      for (int n = 0; n < 4; ++n) kf[0][n] = tile_kf<T::DK>(reinterpret_cast<const char*>(tile), L, 0, n);
#pragma unroll
      for (int ks = 0; ks < T::NKS; ++ks) {
        if (ks + 1 < T::NKS) {
#pragma unroll
          for (int n = 0; n < 4; ++n) kf[(ks + 1) & 1][n] = tile_kf<T::DK>(reinterpret_cast<const char*>(tile), L, ks + 1, n);
        }
#pragma unroll
        for (int n = 0; n < 4; ++n) s[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[ks & 1][n], qf[ks], s[n], 0, 0, 0);
        __builtin_amdgcn_sched_barrier(0);
      }
      float tm = -INFINITY;
      const int kb = k_lo + t * 64 + cq * 4;
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int key = kb + n * 16 + j;
          s[n][j] = (mine && key <= pos && key >= my_lo) ? s[n][j] * sc : -INFINITY;
          tm = fmaxf(tm, s[n][j]);
        }
      tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
      tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
      const float mn = fmaxf(m, tm);
      const float al = mn == -INFINITY ? 1.0f : exp2f(m - mn);
      float ls = 0.0f;
#pragma unroll
      for (int n = 0; n < 4; ++n)
#pragma unroll
        for (int j = 0; j < 4; ++j) { s[n][j] = s[n][j] == -INFINITY ? 0.0f : exp2f(s[n][j] - mn); ls += s[n][j]; }
      ls += __shfl_xor(ls, 16, 64);
      ls += __shfl_xor(ls, 32, 64);
      l = l * al + ls;
      m = mn;
      if (__any(al != 1.0f)) {
#pragma unroll
        for (int i = 0; i < RT; ++i) { o[i][0] *= al; o[i][1] *= al; o[i][2] *= al; o[i][3] *= al; }
      }
      const uint32_t tb = lds_addr(tile);
#pragma unroll
      for (int u = 0; u < 2; ++u) {                       // 32 keys each
        u32x4 pk;
        pk.x = pack2(f2bf(s[2 * u][0]), f2bf(s[2 * u][1])); pk.y = pack2(f2bf(s[2 * u][2]), f2bf(s[2 * u][3]));
        pk.z = pack2(f2bf(s[2 * u + 1][0]), f2bf(s[2 * u + 1][1])); pk.w = pack2(f2bf(s[2 * u + 1][2]), f2bf(s[2 * u + 1][3]));
        const bf16x8 pf = __builtin_bit_cast(bf16x8, pk);
        uint2 f[2][4][2];
        IXT_TILE_VT(f[0], tb, L, 0, u);
#pragma unroll
        for (int gr = 0; gr < RT / 4; ++gr) {             // the next group's reads travel under this one's products
          if (gr + 1 < RT / 4) {
            IXT_TILE_VT(f[(gr + 1) & 1], tb, L, gr + 1, u);
            IXT_TILE_VWAIT(f[gr & 1], 8);
          } else {
            IXT_TILE_VWAIT(f[gr & 1], 0);
          }
#pragma unroll
          for (int i = 0; i < 4; ++i) o[gr * 4 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tile_vfrag(f[gr & 1][i]), pf, o[gr * 4 + i], 0, 0, 0);
        }
      }
    }
  }
  if (!live) return;
  const float inv = l > 0.0f ? 1.0f / l : 0.0f;
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    const float v[4] = {o[i][0] * inv, o[i][1] * inv, o[i][2] * inv, o[i][3] * inv};
    act_store4(a.out, head * a.Rp + row, i * 16 + cq * 4, a.Kp, v);
  }
  const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int c = RT * 16 + cq * 4; c < a.Kp; c += 16) act_store4(a.out, head * a.Rp + row, c, a.Kp, z);
}

// Few rows (decode): a block owns the (at most 16) heads of ONE row and every gridDim.z-th key tile of its window.  Scores: a wave takes 16 of the 64
// keys; P and the tile maxima meet in LDS; output: a wave takes a quarter of the latent columns.  One tile of LDS: two blocks share a CU and one's
// loads run under the other's products.  grid (R, ceil(H / HB), splits), block 256.
template <int RT, int RS>
__global__ __launch_bounds__(256, 2) void k_latent_decode(LatentAttnArgs a) {
  typedef LatentTile<RT, RS> T;
  constexpr int OT = RT / 4;                              // column tiles per wave
  extern __shared__ __attribute__((aligned(16))) bf16_t tile[];
  __shared__ __attribute__((aligned(16))) bf16_t ps[16][72];
  __shared__ float s_m[4][16], s_l[4][16];
  const LatentGeom& g = a.g;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r_in = lane & 15, cq = lane >> 4;
  const int row = blockIdx.x, h0 = blockIdx.y * a.HB, hb = min(a.HB, g.H - h0), nsplit = gridDim.z;
  const int active = a.row_active[row], pos = a.row_pos[row], slot = a.row_slot[row];     // (requested together)
  if (!active) return;
  const bool pair_ok = r_in < hb;
  const int head = h0 + (pair_ok ? r_in : 0);
  const int32_t* prow = a.page_map + (size_t)slot * g.mpg;
  const int k_lo = g.window > 0 ? max(0, pos - g.window + 1) : 0, ntile = (pos - k_lo) / 64 + 1;
  int t = blockIdx.z;
  if (t < ntile) tile_dma<T::DK>(a.pages, cached_row(prow, min(k_lo + t * 64 + lane, pos), a.pshift), tile, wave, lane);
  bf16x8 qf[T::NKS];
#pragma unroll
  for (int ks = 0; ks < RT / 2; ++ks) qf[ks] = latent_q8(a, head * a.Rp + row, ks * 32 + cq * 8);
#pragma unroll
  for (int ks = 0; ks < RS; ++ks)
    qf[RT / 2 + ks] = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(a.qr + ((size_t)row * g.H + head) * g.rotp + ks * 32 + cq * 8));
  f32x4 o[OT];
#pragma unroll
  for (int i = 0; i < OT; ++i) o[i] = f32x4(0.0f);
  float m = -INFINITY, l = 0.0f;                          // l: this lane's keys only
  const float sc = g.scale * 1.44269504088896340736f;
  const TileLane L = tile_lane(r_in, cq);
  [[maybe_unused]] const uint32_t tb = lds_addr(tile) + wave * (OT / 4) * 8192;                              // the wave's first column group
  [[maybe_unused]] const uint32_t tg = lds_addr(tile) + (wave * OT / 4) * 8192;                              // fewer than 4 tiles per wave: the group they are in
  for (; t < ntile; t += nsplit) {
    int off = 0;
    if (t + nsplit < ntile) off = cached_row(prow, min(k_lo + (t + nsplit) * 64 + lane, pos), a.pshift);
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    f32x4 s = f32x4(0.0f);
#pragma unroll
    for (int ks = 0; ks < T::NKS; ++ks) {
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tile_kf<T::DK>(reinterpret_cast<const char*>(tile) + wave * (RS == 1 && ks == RT / 2 ? 1024 : 2048), L, ks, 0), qf[ks], s, 0, 0, 0);
    }
    float tm = -INFINITY;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      s[j] = k_lo + t * 64 + wave * 16 + cq * 4 + j <= pos ? s[j] * sc : -INFINITY;
      tm = fmaxf(tm, s[j]);
    }
    tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
    tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
    if (cq == 0) s_m[wave][r_in] = tm;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(s_m[0][r_in], s_m[1][r_in]), fmaxf(s_m[2][r_in], s_m[3][r_in])));   // (a tile has at least one visible key: finite)
    const float al = exp2f(m - mn);
    float p[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) p[j] = exp2f(s[j] - mn);
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
    for (int u = 0; u < 2; ++u) {                         // lane group q holds keys 32 u + 4 q .. + 3 and 32 u + 16 + 4 q .. + 3 (as in k_latent_attn)
      const uint2 p0 = *reinterpret_cast<const uint2*>(&ps[r_in][u * 32 + 4 * cq]), p1 = *reinterpret_cast<const uint2*>(&ps[r_in][u * 32 + 16 + 4 * cq]);
      u32x4 pv; pv.x = p0.x; pv.y = p0.y; pv.z = p1.x; pv.w = p1.y;
      const bf16x8 pf = __builtin_bit_cast(bf16x8, pv);
      if constexpr (OT >= 4) {                            // whole column groups
        uint2 f[2][4][2];
        IXT_TILE_VT(f[0], tb, L, 0, u);
#pragma unroll
        for (int gr = 0; gr < OT / 4; ++gr) {
          if (gr + 1 < OT / 4) {
            IXT_TILE_VT(f[(gr + 1) & 1], tb, L, gr + 1, u);
            IXT_TILE_VWAIT(f[gr & 1], 8);
          } else {
            IXT_TILE_VWAIT(f[gr & 1], 0);
          }
#pragma unroll
          for (int i = 0; i < 4; ++i) o[gr * 4 + i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tile_vfrag(f[gr & 1][i]), pf, o[gr * 4 + i], 0, 0, 0);
        }
      } else {                                            // OT column tiles, from place (wave OT) % 4 of one group on
        uint2 f[4][2];
        IXT_TILE_VT(f, tg, L, 0, u);
        IXT_TILE_VWAIT(f, 0);
        const int at = (wave * OT) & 3;
#pragma unroll
        for (int i = 0; i < OT; ++i) {
          uint2 x = f[i][0], y = f[i][1];
#pragma unroll
          for (int k = 1; k + i < 4; ++k) {
            const bool take = at == k;
            x.x = take ? f[k + i][0].x : x.x; x.y = take ? f[k + i][0].y : x.y; y.x = take ? f[k + i][1].x : y.x; y.y = take ? f[k + i][1].y : y.y;
          }
          const uint2 xy[2] = {x, y};
          o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tile_vfrag(xy), pf, o[i], 0, 0, 0);
        }
      }
    }
    __syncthreads();                                      // the tile has been read by every wave
    if (t + nsplit < ntile) tile_dma<T::DK>(a.pages, off, tile, wave, lane);
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (cq == 0) s_l[wave][r_in] = l;
  __syncthreads();
  l = (s_l[0][r_in] + s_l[1][r_in]) + (s_l[2][r_in] + s_l[3][r_in]);
  if (!pair_ok) return;
  if (nsplit == 1) {
    const float inv = 1.0f / l;
#pragma unroll
    for (int i = 0; i < OT; ++i) {
      const float v[4] = {o[i][0] * inv, o[i][1] * inv, o[i][2] * inv, o[i][3] * inv};
      act_store4(a.out, head * a.Rp + row, (wave * OT + i) * 16 + cq * 4, a.Kp, v);
    }
    const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (wave == 0)
      for (int c = RT * 16 + cq * 4; c < a.Kp; c += 16) act_store4(a.out, head * a.Rp + row, c, a.Kp, z);
  } else {
    const size_t pi = ((size_t)row * g.H + head) * nsplit + blockIdx.z;
#pragma unroll
    for (int i = 0; i < OT; ++i)
      *reinterpret_cast<float4*>(a.part_o + pi * (RT * 16) + (wave * OT + i) * 16 + cq * 4) = make_float4(o[i][0], o[i][1], o[i][2], o[i][3]);
    if (wave == 0 && cq == 0) { a.part_ml[pi * 2] = m; a.part_ml[pi * 2 + 1] = l; }
  }
}
// Key splits (<= 16) of one (row, head): ml = {maximum, sum} per split -> fac[s] = what split s's weighted sum counts for (threads 0 .. 63 work, all call)
__device__ __forceinline__ void split_factors(const float* __restrict__ ml, int nsplit, int tid, float* fac /*[16] LDS*/) {
  if (tid < 64) {
    const int s = tid & 15;
    const float ms = s < nsplit ? ml[s * 2] : -INFINITY, ls = s < nsplit ? ml[s * 2 + 1] : 0.0f;
    float mm = ms;
#pragma unroll
    for (int off = 1; off < 16; off <<= 1) mm = fmaxf(mm, __shfl_xor(mm, off, 64));
    const float f = ms == -INFINITY ? 0.0f : exp2f(ms - mm);      // a split without a key of its own
    const float ll = row16_sum(ls * f);
    if (tid < 16) fac[s] = f / ll;
  }
  __syncthreads();
}
// four columns of the weighted sums (cols apart per split) put together
__device__ __forceinline__ void split_sum4(const float* __restrict__ o, int cols, int nsplit, const float* fac, float* v) {
  v[0] = v[1] = v[2] = v[3] = 0.0f;
  for (int s0 = 0; s0 < nsplit; s0 += 4) {
    float4 u[4];
#pragma unroll
    for (int s = 0; s < 4; ++s) u[s] = *reinterpret_cast<const float4*>(o + (size_t)min(s0 + s, nsplit - 1) * cols);
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const float f = s0 + s < nsplit ? fac[s0 + s] : 0.0f;
      if (f != 0.0f) { v[0] = fmaf(u[s].x, f, v[0]); v[1] = fmaf(u[s].y, f, v[1]); v[2] = fmaf(u[s].z, f, v[2]); v[3] = fmaf(u[s].w, f, v[3]); }
    }
  }
}
// the key splits of a row's heads put together.  grid (R, H), block 128; nsplit <= 16.
static __global__ __launch_bounds__(128) void k_latent_combine(const float* __restrict__ part_o, const float* __restrict__ part_ml, int nsplit, int cols, int H, int Rp,
                                                        const int32_t* __restrict__ row_active, bf16_t* __restrict__ out, int Kp) {
  __shared__ float fac[16];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  if (!row_active[r]) return;
  const size_t p0 = ((size_t)r * H + h) * nsplit;
  split_factors(part_ml + p0 * 2, nsplit, tid, fac);
  for (int c = tid * 4; c < Kp; c += 512) {
    float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (c < cols) split_sum4(part_o + p0 * cols + c, cols, nsplit, fac, v);
    act_store4(out, h * Rp + r, c, Kp, v);
  }
}
// head-major slices (row h Rp + r, n columns each) -> act of the output projection: column h n + c, times sigmoid of gate column g0 + h n + c (gate.n ==
// 0: none).  grid (R, ceil(Kp / 256)), block 256.
template <typename T>
__global__ __launch_bounds__(256) void k_heads_x(Slices t, int H, int n, int Rp, Slices gate, int g0, T* __restrict__ out, int Kp) {
  const int r = blockIdx.x, k = blockIdx.y * 256 + threadIdx.x;
  if (k >= Kp) return;
  float v = 0.0f;
  if (k < H * n) {
    v = t.at((k / n) * Rp + r, k % n);
    if (gate.n > 0) v *= f32_sigmoid(gate.at(r, g0 + k));
  }
  act_store1(out, r, k, Kp, v);
}

// ---------------------------------------------------------------------------------------------------- gated delta rule
struct DeltaGeom {
  int H, KH, d, dv, dp, taps;               // heads, query/key heads, key dims, value dims, padded key dims (16 RP), convolution taps
  int oq, ok, ov, ob, oa, og, ra, rg;       // columns of the input projection: q, k, v, beta, decay rank, gate rank; the two ranks
  int og2;                                  // column of the output gate in the second low-rank product (decays start at 0)
  int C;                                    // convolution channels = 2 KH d + H dv (q, k, v)
};
// the two low-rank activations side by side as ONE operand (the second matrices form a block diagonal).  grid R, block 128.
template <typename T>
__global__ __launch_bounds__(128) void k_lowrank_x(Slices t, DeltaGeom g, T* __restrict__ out, int Kp) {
  const int r = blockIdx.x;
  for (int k = threadIdx.x; k < Kp; k += 128) {
    float v = 0.0f;
    if (k < g.ra) v = t.at(r, g.oa + k);
    else if (k < g.ra + g.rg) v = t.at(r, g.og + k - g.ra);
    act_store1(out, r, k, Kp, v);
  }
}

// one channel of a short causal convolution: taps[0 .. n-1], the last for the row itself.  Earlier inputs come from the segment's rows or, before
// its start, from the group's tail (oldest first).  Returns the convolution and leaves the channel's next tail (rows among the segment's last
// n - 1 write their input; the last row carries older entries over when the segment is shorter than the tail).
struct ConvCtx { const float* tail_in; float* tail_out; int j, n, start; };      // tail_out nullptr: another block leaves the tail
__device__ __forceinline__ float conv_channel(const Slices& t, int r, int col, const float* __restrict__ tp, int taps, int ch, int C, const ConvCtx& cc) {
  const float x0 = t.at(r, col);
  float acc = x0 * tp[taps - 1];
  for (int b0 = 1; b0 < taps; b0 += 4) {                   // four earlier inputs in flight
    float v[4], w[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int b = min(b0 + i, taps - 1);
      const bool mine = cc.j - b >= 0;
      const float* src = mine ? t.p + (size_t)(r - b) * t.ncols + col : cc.tail_in + (size_t)(taps - 1 - (b - cc.j)) * C + ch;
      v[i] = mine || cc.start > 0 ? *src : 0.0f;
      w[i] = b0 + i < taps ? tp[taps - 1 - b] : 0.0f;
      if (mine)
        for (int s = 1; s < t.n; ++s) v[i] += src[(size_t)s * t.stride];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) acc = fmaf(v[i], w[i], acc);
  }
  if (cc.tail_out == nullptr) return acc;
  const int dist = cc.n - 1 - cc.j;
  if (dist < taps - 1) cc.tail_out[(size_t)(taps - 2 - dist) * C + ch] = x0;
  if (dist == 0)
    for (int e = cc.n; e < taps - 1; ++e)      // entries that are still older than the segment
      cc.tail_out[(size_t)(taps - 2 - e) * C + ch] = cc.start > 0 ? cc.tail_in[(size_t)(taps - 2 - (e - cc.n)) * C + ch] : 0.0f;
  return acc;
}

// Everything the recurrence takes in: convolutions, silu, unit vectors, step sizes, decays (f32).  wave = one query/key head, or one value head with
// its beta and decays.  grid (R, ceil((KH + H) / 4)), block 256.
struct DeltaPrepArgs {
  Slices t, t2; DeltaGeom g;
  const float *cq, *ck, *cv, *a_log, *dt_bias;
  const int32_t *row_seg, *row_j, *seg;
  float* tails;                             // [group][2][taps - 1][C]
  float *q, *k, *kq, *v, *dec, *beta;       // [R][KH][dp], .., [R][KH], [R][H][dv], [R][H][dp], [R][H]
};
static __global__ __launch_bounds__(256) void k_delta_prep(DeltaPrepArgs a) {
  const DeltaGeom& g = a.g;
  const int r = blockIdx.x, lane = threadIdx.x & 63, vi = blockIdx.y * 4 + (threadIdx.x >> 6);
  const int s = a.row_seg[r];
  if (s < 0 || vi >= g.KH + g.H) return;
  const int32_t* sg = a.seg + (size_t)s * 8;
  const size_t tsz = (size_t)(g.taps - 1) * g.C;
  float* tb = a.tails + (size_t)sg[2] * 2 * tsz;
  const ConvCtx cc{tb + (size_t)sg[4] * tsz, tb + (size_t)(sg[4] ^ 1) * tsz, a.row_j[r], sg[1], sg[3]};
  if (vi < g.KH) {
    float* qo = a.q + ((size_t)r * g.KH + vi) * g.dp;
    float* ko = a.k + ((size_t)r * g.KH + vi) * g.dp;
    float qq = 0.0f, kk = 0.0f, qk = 0.0f;
    float qv[8], kv[8];                     // dims up to 512, eight per lane
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int c = lane + 64 * i;
      qv[i] = kv[i] = 0.0f;
      if (c < g.d) {
        const int ch = vi * g.d + c;
        const float x = conv_channel(a.t, r, g.oq + ch, a.cq + (size_t)ch * g.taps, g.taps, ch, g.C, cc);
        const float y = conv_channel(a.t, r, g.ok + ch, a.ck + (size_t)ch * g.taps, g.taps, g.KH * g.d + ch, g.C, cc);
        qv[i] = x * f32_sigmoid(x); kv[i] = y * f32_sigmoid(y);
        qq = fmaf(qv[i], qv[i], qq); kk = fmaf(kv[i], kv[i], kk);
      }
    }
    qq = wave_sum(qq); kk = wave_sum(kk);
    const float qs = 1.0f / sqrtf(qq + 1e-6f) * (1.0f / sqrtf((float)g.d)), ks = 1.0f / sqrtf(kk + 1e-6f);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int c = lane + 64 * i;
      if (c < g.dp) { qo[c] = qv[i] * qs; ko[c] = kv[i] * ks; qk = fmaf(qv[i] * qs, kv[i] * ks, qk); }
    }
    qk = wave_sum(qk);
    if (lane == 0) a.kq[(size_t)r * g.KH + vi] = qk;
    return;
  }
  const int h = vi - g.KH;
  for (int c = lane; c < g.dv; c += 64) {
    const int ch = h * g.dv + c;
    const float x = conv_channel(a.t, r, g.ov + ch, a.cv + (size_t)ch * g.taps, g.taps, 2 * g.KH * g.d + ch, g.C, cc);
    a.v[((size_t)r * g.H + h) * g.dv + c] = x * f32_sigmoid(x);
  }
  const float ea = expf(a.a_log[h]);
  float* go = a.dec + ((size_t)r * g.H + h) * g.dp;
  for (int c = lane; c < g.dp; c += 64)
    go[c] = c < g.d ? expf(-ea * f32_softplus(a.t2.at(r, h * g.d + c) + a.dt_bias[h * g.d + c])) : 0.0f;
  if (lane == 0) a.beta[(size_t)r * g.H + h] = f32_sigmoid(a.t.at(r, g.ob + h));
}

// The recurrence, per head:  S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q, all f32.  The columns of S (value dims) never meet, so a
// block owns 16 of them for one (segment, head): a wave four, 16 lanes per column with RP key rows each in registers.  o = (g S)^T q + (k . q) u: both
// sums over the key rows are taken from the decayed state and run side by side.  q, k and the decays of TT tokens at a time come by LDS-DMA into one of
// two buffers while the other is used; a token's operands are read into registers one token ahead.
// State [group][H][dv][dp]; a segment at position 0 starts from zero.  grid (segments, H, ceil(dv / 16)), block 256, LDS 2 x 3 x TT x DP floats.
struct DeltaScanArgs {
  DeltaGeom g;
  const int32_t *seg, *nseg;
  const float *q, *k, *kq, *v, *dec, *beta;
  float* state;
  float* o;                                 // [R][H][dv]
};
// key row of register i of lane `sub`: 16 lanes x 4 rows per access, so that 16 lanes read and write 256 contiguous bytes
template <int RP> __device__ __forceinline__ int delta_row(int sub, int i) { return RP >= 4 ? (i >> 2) * 64 + sub * 4 + (i & 3) : sub * RP + i; }
template <int RP> constexpr int scan_tokens() { return RP <= 8 ? 16 : 128 / RP; }
template <int RP>
__global__ __launch_bounds__(256) void k_delta_scan(DeltaScanArgs a) {
  constexpr int DP = 16 * RP, TT = scan_tokens<RP>(), TILE = 3 * TT * DP, NW = TILE / 256;      // floats of a token tile; wave loads (64 x 16 bytes) in it
  static_assert(TILE % 256 == 0, "whole wave loads");
  extern __shared__ __attribute__((aligned(16))) float sm[];            // [2][q, k, decay][TT][DP]
  __shared__ float sv[2][TT][16], sb[2][TT], skq[2][TT], so[TT][16];
  const DeltaGeom& g = a.g;
  const int s = blockIdx.x;
  if (s >= *a.nseg) return;
  const int first = a.seg[s * 8], n = a.seg[s * 8 + 1], grp = a.seg[s * 8 + 2], start = a.seg[s * 8 + 3];
  if (n <= 0) return;
  const int h = blockIdx.y, kh = h / (g.H / g.KH), tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, sub = lane & 15;
  const int cb = blockIdx.z * 16, cl = wave * 4 + (lane >> 4), col = cb + cl;
  const bool col_ok = col < g.dv;
  float S[RP];
  float* sp = a.state + (((size_t)grp * g.H + h) * g.dv + (col_ok ? col : 0)) * DP;
#pragma unroll
  for (int i = 0; i < RP; ++i) S[i] = 0.0f;
  if (start > 0 && col_ok) {
#pragma unroll
    for (int i = 0; i < RP; ++i) S[i] = sp[delta_row<RP>(sub, i)];
  }
#pragma unroll
  for (int i = 0; i < RP; ++i) asm volatile("" : "+v"(S[i]));        // arrived before the loop: nothing in it waits for HBM
  float pv = 0.0f, pb = 0.0f;
  const int vt = tid >> 4, vc = cb + (tid & 15);
  // tokens T0_ .. T0_ + TT - 1 (past the end: the last one again, never used): vectors into buffer B_, scalars into registers
#define IXT_SCAN_FETCH(T0_, B_)                                                                                                         \
  do {                                                                                                                                  \
    _Pragma("unroll") for (int i_ = 0; i_ < (NW + 3) / 4; ++i_) {                                                                       \
      const int w_ = i_ * 4 + wave;                                                                                                     \
      if (NW % 4 == 0 || w_ < NW) {                                                                                                     \
        const int e_ = w_ * 256 + lane * 4, x_ = e_ / (TT * DP), t_ = (e_ / DP) % TT, c_ = e_ % DP, r_ = first + min((T0_) + t_, n - 1); \
        const float* src_ = x_ == 0 ? a.q + ((size_t)r_ * g.KH + kh) * DP : (x_ == 1 ? a.k + ((size_t)r_ * g.KH + kh) * DP : a.dec + ((size_t)r_ * g.H + h) * DP); \
        __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(src_ + c_),                                    \
                                         (__attribute__((address_space(3))) void*)(sm + (B_) * TILE + w_ * 256), 16, 0, 0);              \
      }                                                                                                                                 \
    }                                                                                                                                   \
    if (vt < TT) pv = vc < g.dv ? a.v[((size_t)(first + min((T0_) + vt, n - 1)) * g.H + h) * g.dv + vc] : 0.0f;                         \
    if (tid < TT) pb = a.beta[(size_t)(first + min((T0_) + tid, n - 1)) * g.H + h];                                                     \
    else if (tid < 2 * TT) pb = a.kq[(size_t)(first + min((T0_) + tid - TT, n - 1)) * g.KH + kh];                                       \
  } while (0)
  IXT_SCAN_FETCH(0, 0);
  int buf = 0;
  for (int t0 = 0; t0 < n; t0 += TT, buf ^= 1) {
    if (vt < TT) sv[buf][vt][tid & 15] = pv;
    if (tid < TT) sb[buf][tid] = pb;
    else if (tid < 2 * TT) skq[buf][tid - TT] = pb;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();                                        // this tile is in LDS; the read-outs of the one before have left
    if (t0 + TT < n) IXT_SCAN_FETCH(t0 + TT, buf ^ 1);
    const int nt = min(TT, n - t0);
    const float* qb = sm + buf * TILE;
#define IXT_SCAN_LOAD(X_, T_)                                                                                                       \
  do {                                                                                                                              \
    const int tt_ = min((T_), TT - 1);                                                                                              \
    _Pragma("unroll") for (int i_ = 0; i_ < RP; ++i_) {                                                                             \
      const int e_ = tt_ * DP + delta_row<RP>(sub, i_);                                                                             \
      q##X_[i_] = qb[e_]; k##X_[i_] = qb[TT * DP + e_]; g##X_[i_] = qb[2 * TT * DP + e_];                                           \
    }                                                                                                                               \
    v##X_ = sv[buf][tt_][cl]; b##X_ = sb[buf][tt_]; d##X_ = skq[buf][tt_];                                                          \
  } while (0)
#define IXT_SCAN_STEP(X_, T_)                                                                                                       \
  do {                                                                                                                              \
    float a0_ = 0.0f, a1_ = 0.0f, b0_ = 0.0f, b1_ = 0.0f;                                                                           \
    _Pragma("unroll") for (int i_ = 0; i_ < RP; ++i_) {                                                                             \
      S[i_] *= g##X_[i_];                                                                                                           \
      if (i_ & 1) { a1_ = fmaf(k##X_[i_], S[i_], a1_); b1_ = fmaf(q##X_[i_], S[i_], b1_); }                                         \
      else { a0_ = fmaf(k##X_[i_], S[i_], a0_); b0_ = fmaf(q##X_[i_], S[i_], b0_); }                                                \
    }                                                                                                                               \
    const float ax_ = row16_sum(a0_ + a1_), bx_ = row16_sum(b0_ + b1_), u_ = b##X_ * (v##X_ - ax_);                                 \
    _Pragma("unroll") for (int i_ = 0; i_ < RP; ++i_) S[i_] = fmaf(k##X_[i_], u_, S[i_]);                                           \
    if (sub == 0) so[T_][cl] = fmaf(d##X_, u_, bx_);                                                                                \
  } while (0)
    float qA[RP], kA[RP], gA[RP], vA, bA, dA, qB[RP], kB[RP], gB[RP], vB, bB, dB;
    IXT_SCAN_LOAD(A, 0);
    for (int t = 0; t < nt; t += 2) {
      IXT_SCAN_LOAD(B, t + 1);
      IXT_SCAN_STEP(A, t);
      if (t + 1 < nt) {
        IXT_SCAN_LOAD(A, t + 2);
        IXT_SCAN_STEP(B, t + 1);
      }
    }
#undef IXT_SCAN_LOAD
#undef IXT_SCAN_STEP
    __syncthreads();                                        // read-outs of the tile -> HBM, 16 consecutive columns per token
    if (vt < nt && vc < g.dv) a.o[((size_t)(first + t0 + vt) * g.H + h) * g.dv + vc] = so[vt][tid & 15];
  }
#undef IXT_SCAN_FETCH
  if (col_ok) {
#pragma unroll
    for (int i = 0; i < RP; ++i) sp[delta_row<RP>(sub, i)] = S[i];
  }
}

// One token per row (decode): everything between the projections of a gated-delta layer in one launch.  Block = (row, head): its whole state matrix is
// requested first and travels while the convolutions, unit vectors, decays and the step size are computed; then the recurrence on 16 columns at a
// time, the head's norm and output gate.  A query / key head that several heads share is computed by each of them; the first one keeps its tail.
// grid (R, H), block 256, dynamic LDS = (3 dp + 2 dv) floats.
struct DeltaStepArgs {
  Slices t, t2; DeltaGeom g;
  const float *cq, *ck, *cv, *a_log, *dt_bias, *nw;
  float eps;
  const int32_t *row_active, *row_slot, *row_pos, *parity;     // parity: as k_segments has left it for the NEXT pass
  float *tails, *state;
};
template <typename T, int RP>
__global__ __launch_bounds__(256) void k_delta_step(DeltaStepArgs a, T* __restrict__ out, int Kp) {
  constexpr int DP = 16 * RP, NJ = RP <= 8 ? 8 : (RP == 16 ? 4 : 2);      // columns in flight per lane
  extern __shared__ __attribute__((aligned(16))) float lm[];
  __shared__ float red[4], red2[4];
  float *qs = lm, *ks = lm + DP, *gs = lm + 2 * DP, *vs = lm + 3 * DP, *os = vs + a.g.dv;
  const DeltaGeom& g = a.g;
  const int r = blockIdx.x, h = blockIdx.y, kh = h / (g.H / g.KH), tid = threadIdx.x, lane = tid & 63, sub = lane & 15, cl = (tid >> 6) * 4 + (lane >> 4);
  const int active = a.row_active[r], grp = a.row_slot[r], start = a.row_pos[r];      // (requested together)
  if (!active) return;
  const int par = a.parity[grp] ^ 1;
  float* sp = a.state + ((size_t)grp * g.H + h) * g.dv * DP;
  float S[NJ][RP];
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int col = cl + 16 * j;
#pragma unroll
    for (int i = 0; i < RP; ++i) S[j][i] = (start > 0 && col < g.dv) ? sp[(size_t)col * DP + delta_row<RP>(sub, i)] : 0.0f;
  }
  const size_t tsz = (size_t)(g.taps - 1) * g.C;
  float* tb = a.tails + (size_t)grp * 2 * tsz;
  const float* tail_in = tb + (size_t)par * tsz;
  float* tail_out = tb + (size_t)(par ^ 1) * tsz;
  const float gate0 = tid < g.dv ? a.t2.at(r, g.og2 + h * g.dv + tid) : 0.0f, beta_z = a.t.at(r, g.ob + h), ea = expf(a.a_log[h]);
  const bool first = h % (g.H / g.KH) == 0;          // of the heads that share a query / key head
  float qq = 0.0f, kk = 0.0f;
  // one channel per thread and round: queries, keys, decays, values side by side
  for (int i = tid; i < 3 * DP + g.dv; i += 256) {
    const int kind = i < DP ? 0 : (i < 2 * DP ? 1 : (i < 3 * DP ? 2 : 3)), c = i - kind * DP;
    float x = 0.0f;
    if (kind == 2) {
      if (c < g.d) x = expf(-ea * f32_softplus(a.t2.at(r, h * g.d + c) + a.dt_bias[h * g.d + c]));
    } else if (kind == 3 || c < g.d) {
      const int ch = kind == 3 ? h * g.dv + c : kh * g.d + c, col = (kind == 0 ? g.oq : (kind == 1 ? g.ok : g.ov)) + ch;
      x = conv_channel(a.t, r, col, (kind == 0 ? a.cq : (kind == 1 ? a.ck : a.cv)) + (size_t)ch * g.taps, g.taps, kind == 3 ? 2 * g.KH * g.d + ch : kind * g.KH * g.d + ch, g.C,
                       ConvCtx{tail_in, kind == 3 || first ? tail_out : nullptr, 0, 1, start});
      x *= f32_sigmoid(x);
      if (kind == 0) qq = fmaf(x, x, qq);
      else if (kind == 1) kk = fmaf(x, x, kk);
    }
    lm[i] = x;                              // [q | k | decay | v]
  }
  const float beta = f32_sigmoid(beta_z);
  qq = wave_sum(qq); kk = wave_sum(kk);
  if (lane == 0) { red[tid >> 6] = qq; red2[tid >> 6] = kk; }
  __syncthreads();
  const float qn = 1.0f / sqrtf((red[0] + red[1]) + (red[2] + red[3]) + 1e-6f) * (1.0f / sqrtf((float)g.d)), kn = 1.0f / sqrtf((red2[0] + red2[1]) + (red2[2] + red2[3]) + 1e-6f);
  float qv[RP], kv[RP], gv[RP], qk = 0.0f;
#pragma unroll
  for (int i = 0; i < RP; ++i) {
    const int e = delta_row<RP>(sub, i);
    qv[i] = qs[e] * qn; kv[i] = ks[e] * kn; gv[i] = gs[e];
    qk = fmaf(qv[i], kv[i], qk);
  }
  qk = row16_sum(qk);
  for (int c0 = 0; c0 < g.dv; c0 += 16 * NJ) {
    if (c0 > 0) {
#pragma unroll
      for (int j = 0; j < NJ; ++j) {
        const int col = c0 + cl + 16 * j;
#pragma unroll
        for (int i = 0; i < RP; ++i) S[j][i] = (start > 0 && col < g.dv) ? sp[(size_t)col * DP + delta_row<RP>(sub, i)] : 0.0f;
      }
    }
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      const int col = c0 + cl + 16 * j;
      float ax = 0.0f, bx = 0.0f;
#pragma unroll
      for (int i = 0; i < RP; ++i) { S[j][i] *= gv[i]; ax = fmaf(kv[i], S[j][i], ax); bx = fmaf(qv[i], S[j][i], bx); }
      ax = row16_sum(ax);
      bx = row16_sum(bx);
      if (col < g.dv) {
        const float u = beta * (vs[col] - ax);
#pragma unroll
        for (int i = 0; i < RP; ++i) sp[(size_t)col * DP + delta_row<RP>(sub, i)] = fmaf(kv[i], u, S[j][i]);
        if (sub == 0) os[col] = fmaf(qk, u, bx);
      }
    }
  }
  __syncthreads();
  float ss = 0.0f;
  for (int c = tid; c < g.dv; c += 256) ss = fmaf(os[c], os[c], ss);
  const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)g.dv + a.eps);
  for (int c = tid; c < g.dv; c += 256) act_store1(out, r, h * g.dv + c, Kp, os[c] * rs * a.nw[c] * f32_sigmoid(c < 256 ? gate0 : a.t2.at(r, g.og2 + h * g.dv + c)));
  if (h == g.H - 1)
    for (int k = g.H * g.dv + tid; k < Kp; k += 256) act_store1(out, r, k, Kp, 0.0f);
}

// read-out: o / rms(o) * norm * sigmoid(gate) per head -> the output projection's operand (column h dv + c).  grid (R, ceil(H / 4)), block 256.
template <typename T>
__global__ __launch_bounds__(256) void k_delta_out(const float* __restrict__ o, Slices t2, DeltaGeom g, const float* __restrict__ nw, float eps, const int32_t* __restrict__ row_seg,
                                                   T* __restrict__ out, int Kp) {
  const int r = blockIdx.x, h = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (h >= g.H) return;
  const bool live = row_seg[r] >= 0;
  const float* oh = o + ((size_t)r * g.H + h) * g.dv;
  float ss = 0.0f;
  if (live)
    for (int c = lane; c < g.dv; c += 64) ss = fmaf(oh[c], oh[c], ss);
  const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)g.dv + eps);
  for (int c = lane; c < g.dv; c += 64)
    act_store1(out, r, h * g.dv + c, Kp, live ? oh[c] * rs * nw[c] * f32_sigmoid(t2.at(r, g.og2 + h * g.dv + c)) : 0.0f);
  if (h == g.H - 1)
    for (int k = g.H * g.dv + lane; k < Kp; k += 64) act_store1(out, r, k, Kp, 0.0f);
}

// ---------------------------------------------------------------------------------------------------- feed-forward
// gated unit (kind: IXT_GLU_*) from interleaved slices (tile 2 j gate, 2 j + 1 up).  grid (rows, ceil(Fp / 256)), block 256; rb_exp: rows of blocks
// without an expert are skipped.
template <typename T>
__global__ __launch_bounds__(256) void k_glu_slices(Slices t, int Fp, int kind, float limit, T* __restrict__ out, const int32_t* __restrict__ rb_exp) {
  const int f = blockIdx.y * 256 + threadIdx.x, r = blockIdx.x;
  if (f >= Fp || (rb_exp != nullptr && rb_exp[r >> 4] < 0)) return;
  const int c = (f >> 4) * 32 + (f & 15);
  act_store1(out, r, f, Fp, ixt_glu(kind, t.at(r, c), t.at(r, c + 16), limit));
}

// the same for a unit without a gate.  grid (rows, ceil(Fp / 256)), block 256
template <typename T>
__global__ __launch_bounds__(256) void k_act_slices(Slices t, int Fp, int kind, const float* __restrict__ par, T* __restrict__ out, const int32_t* __restrict__ rb_exp) {
  const int f = blockIdx.y * 256 + threadIdx.x, r = blockIdx.x;
  if (f >= Fp || (rb_exp != nullptr && rb_exp[r >> 4] < 0)) return;
  const float u = t.at(r, f);
  if (kind == IXT_ACT_XIELU) {                              // (no hardware functions here: the 32-bit mode)
    const float n = fminf(u, 0.0f), p = fmaxf(u, 0.0f);
    act_store1(out, r, f, Fp, fmaf(0.5f, u, fmaf(par[0] * p, p, par[1] * (expm1f(n) - n))));
  } else act_store1(out, r, f, Fp, ixt_act(kind, u, par));
}
// the numbers of an xIELU unit from its tensor: par = {softplus(p), 1/2 + softplus(q)}
static __global__ void k_xielu_numbers(const float* __restrict__ act, float* __restrict__ par) {
  if (threadIdx.x == 0) { par[0] = f32_softplus(act[0]); par[1] = 0.5f + f32_softplus(act[1]); }
}

// The choice of experts for a row.  IXT_ROUTE_SOFTMAX: scores s = softmax over all n logits; IXT_ROUTE_SIGMOID: s = sigmoid(z); IXT_ROUTE_CHOSEN: s = z.
// The `top` largest s + corr (first index on a tie), inside the `keep` of `groups` equal groups of neighbours whose two largest s + corr add up to most;
// weights are the picked s (CHOSEN: the softmax over the picked ones), divided by (their sum + 1e-20) if norm, times scale.
// Logits are products plus bias[e] (nullptr: none).  gate: one more row of the router's matrix behind the experts, whose sigmoid goes to gate[row].
struct RouteRule { int n, top, kind, groups, keep, norm; float scale; const float *corr, *bias; float* gate; };
// one wave; z [n] in LDS (overwritten: choice scores), gs [2 groups] in LDS; n <= 1024
__device__ __forceinline__ void route_top(float* z, float* gs, const RouteRule& a, int lane, int32_t* idx, float* wts) {
  const int n = a.n;
  float v[16], mx = -INFINITY, sum = 1.0f;
#pragma unroll
  for (int i = 0; i < 16; ++i) v[i] = lane + 64 * i < n ? z[lane + 64 * i] : -INFINITY;
  if (a.kind == IXT_ROUTE_SOFTMAX) {
#pragma unroll
    for (int i = 0; i < 16; ++i) mx = fmaxf(mx, v[i]);
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) mx = fmaxf(mx, __shfl_xor(mx, off, 64));
    sum = 0.0f;
#pragma unroll
    for (int i = 0; i < 16; ++i) if (lane + 64 * i < n) sum += expf(v[i] - mx);
    sum = wave_sum(sum);
  }
  float s[16];                                             // scores; v becomes the choice scores
#pragma unroll
  for (int i = 0; i < 16; ++i) {
    const int e = lane + 64 * i;
    s[i] = 0.0f;
    if (e < n) {
      s[i] = a.kind == IXT_ROUTE_SOFTMAX ? expf(v[i] - mx) / sum : a.kind == IXT_ROUTE_SIGMOID ? f32_sigmoid(v[i]) : v[i];
      v[i] = a.corr != nullptr ? s[i] + a.corr[e] : s[i];
    }
  }
  if (a.groups > 1) {                                      // closed groups: minus infinity
    const int size = n / a.groups;
#pragma unroll
    for (int i = 0; i < 16; ++i) if (lane + 64 * i < n) z[lane + 64 * i] = v[i];
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    for (int g = lane; g < a.groups; g += 64) {
      float b1 = -INFINITY, b2 = -INFINITY;
      for (int e = 0; e < size; ++e) {
        const float c = z[g * size + e];
        b2 = fmaxf(b2, fminf(b1, c));
        b1 = fmaxf(b1, c);
      }
      gs[g] = size > 1 ? b1 + b2 : b1;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    for (int g = lane; g < a.groups; g += 64) {            // open if fewer than `keep` groups come before it
      int before = 0;
      for (int o = 0; o < a.groups; ++o) before += gs[o] > gs[g] || (gs[o] == gs[g] && o < g) ? 1 : 0;
      gs[a.groups + g] = before < a.keep ? 1.0f : 0.0f;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if (lane + 64 * i < n && gs[a.groups + (lane + 64 * i) / size] == 0.0f) v[i] = -INFINITY;
  }
  float total = 0.0f;
  for (int j = 0; j < a.top; ++j) {
    float b = -INFINITY;
    int bi = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if (v[i] > b) { b = v[i]; bi = lane + 64 * i; }
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const float ob = __shfl_xor(b, off, 64);
      const int oi = __shfl_xor(bi, off, 64);
      if (ob > b || (ob == b && oi < bi)) { b = ob; bi = oi; }
    }
    if (bi >= n) bi = 0;                                   // only a row without finite scores gets here: any expert will do
    float w = 0.0f;
#pragma unroll
    for (int i = 0; i < 16; ++i) if (lane + 64 * i == bi) { v[i] = -INFINITY; w = s[i]; }
    w = __shfl(w, bi & 63, 64);
    if (a.kind == IXT_ROUTE_CHOSEN) {                      // relative to the first, the largest
      if (j == 0) mx = w;
      w = expf(w - mx);
    }
    total += w;
    if (lane == 0) { idx[j] = bi; wts[j] = w; }
  }
  const bool divide = a.norm || a.kind == IXT_ROUTE_CHOSEN;
  const float f = divide ? a.scale / (total + 1e-20f) : a.scale;
  if (lane == 0 && (divide || a.scale != 1.0f))
    for (int j = 0; j < a.top; ++j) wts[j] *= f;
}
// router: logits (f32 residual x f32 weights) and choice of RB rows in one block, NE experts at a time: a thread takes every 256th feature (every 256th group
// of four where rows start on 16 bytes) of the RB rows and the NE weight rows.  w [n (+ 1)][Ep]; grid ceil(R / RB), block 256, LDS RB (n + 2 groups) floats.
template <int RB, int NE>
__global__ __launch_bounds__(256) void k_route(const float* __restrict__ x, const float* __restrict__ w, int E, int Ep, RouteRule rule, int R, int32_t* __restrict__ idx,
                                               float* __restrict__ wts) {
  extern __shared__ __attribute__((aligned(16))) float z[];            // [RB][n], [RB][2 groups]
  __shared__ float red[4][RB * NE];
  const int n = rule.n, nw = n + (rule.gate != nullptr ? 1 : 0), row = rule.top;
  const int r0 = blockIdx.x * RB, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const float* xr[RB];
#pragma unroll
  for (int i = 0; i < RB; ++i) xr[i] = x + (size_t)min(r0 + i, R - 1) * E;
  for (int e0 = 0; e0 < nw; e0 += NE) {
    float acc[RB][NE];
#pragma unroll
    for (int i = 0; i < RB; ++i)
#pragma unroll
      for (int e = 0; e < NE; ++e) acc[i][e] = 0.0f;
    const float* wr[NE];
#pragma unroll
    for (int e = 0; e < NE; ++e) wr[e] = w + (size_t)min(e0 + e, nw - 1) * Ep;
    if ((E & 3) == 0) {
      for (int k = tid * 4; k < E; k += 1024) {
        float4 xv[RB], wv[NE];
#pragma unroll
        for (int i = 0; i < RB; ++i) xv[i] = *reinterpret_cast<const float4*>(xr[i] + k);
#pragma unroll
        for (int e = 0; e < NE; ++e) wv[e] = *reinterpret_cast<const float4*>(wr[e] + k);
#pragma unroll
        for (int i = 0; i < RB; ++i)
#pragma unroll
          for (int e = 0; e < NE; ++e) acc[i][e] = fmaf(xv[i].x, wv[e].x, fmaf(xv[i].y, wv[e].y, fmaf(xv[i].z, wv[e].z, fmaf(xv[i].w, wv[e].w, acc[i][e]))));
      }
    } else {
      for (int k = tid; k < E; k += 256) {
        float xv[RB], wv[NE];
#pragma unroll
        for (int i = 0; i < RB; ++i) xv[i] = xr[i][k];
#pragma unroll
        for (int e = 0; e < NE; ++e) wv[e] = wr[e][k];
#pragma unroll
        for (int i = 0; i < RB; ++i)
#pragma unroll
          for (int e = 0; e < NE; ++e) acc[i][e] = fmaf(xv[i], wv[e], acc[i][e]);
      }
    }
#pragma unroll
    for (int i = 0; i < RB; ++i)
#pragma unroll
      for (int e = 0; e < NE; ++e) {
        const float t = wave_sum(acc[i][e]);
        if (lane == 0) red[wave][i * NE + e] = t;
      }
    __syncthreads();
    if (tid < RB * NE && e0 + tid % NE < nw) {
      const int e = e0 + tid % NE, i = tid / NE;
      const float v = (red[0][tid] + red[1][tid]) + (red[2][tid] + red[3][tid]);
      if (e < n) z[i * n + e] = rule.bias != nullptr ? v + rule.bias[e] : v;
      else if (r0 + i < R) rule.gate[r0 + i] = f32_sigmoid(v);
    }
    __syncthreads();
  }
  for (int i = wave; i < RB; i += 4)
    if (r0 + i < R) route_top(z + (size_t)i * n, z + (size_t)RB * n + i * 2 * rule.groups, rule, lane, idx + (size_t)(r0 + i) * row, wts + (size_t)(r0 + i) * row);
}
// any number of experts (<= 1024): destination row of every copy by one pass of counters; the order inside an expert is free.  One block of 1024.
static __global__ __launch_bounds__(1024) void k_moe_plan_any(const int32_t* __restrict__ idx, int npairs, int n, int align, int nrb_cap, int32_t* __restrict__ pos, int32_t* __restrict__ rb_exp) {
  __shared__ int cnt[1024], off[1024];
  const int tid = threadIdx.x;
  cnt[tid] = 0;
  for (int i = tid; i < nrb_cap; i += 1024) rb_exp[i] = -1;
  __syncthreads();
  for (int p = tid; p < npairs; p += 1024) pos[p] = atomicAdd(&cnt[idx[p]], 1);
  __syncthreads();
  const int padded = tid < n ? (cnt[tid] + align - 1) / align * align : 0;
  off[tid] = padded;
  __syncthreads();
  for (int o = 1; o < 1024; o <<= 1) {
    const int v = tid >= o ? off[tid - o] : 0;
    __syncthreads();
    off[tid] += v;
    __syncthreads();
  }
  const int base = off[tid] - padded;
  __syncthreads();
  off[tid] = base;
  __syncthreads();
  if (tid < n)
    for (int i = 0; i < (cnt[tid] + 15) / 16; ++i) rb_exp[base / 16 + i] = tid;
  for (int p = tid; p < npairs; p += 1024) pos[p] += off[idx[p]];
}
static __global__ __launch_bounds__(256) void k_gather32(const float* __restrict__ x, const int32_t* __restrict__ pos, int top, int Ep, float* __restrict__ xg) {
  const int k = blockIdx.y * 256 + threadIdx.x, p = blockIdx.x;
  if (k < Ep) xg[(size_t)pos[p] * Ep + k] = x[(size_t)(p / top) * Ep + k];
}
// few rows whose expert outputs lie in many split-K slices: the weighted sum of a row's copies as one slice.  grid (ceil(ncols / 256), R), block 64.
static __global__ __launch_bounds__(64) void k_moe_sum(Slices t, const int32_t* __restrict__ pos, const float* __restrict__ wts, int top, float* __restrict__ out) {
  const int c = (blockIdx.x * 64 + threadIdx.x) * 4, r = blockIdx.y;
  if (c >= t.ncols) return;
  float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int j = 0; j < top; ++j) {
    float u[4];
    t.at4(pos[(size_t)r * top + j], c, u);
    const float w = wts[(size_t)r * top + j];
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = fmaf(w, u[i], v[i]);
  }
  *reinterpret_cast<float4*>(out + (size_t)r * t.ncols + c) = make_float4(v[0], v[1], v[2], v[3]);
}
