// ixt_retention_kernels.h -- retention (IXT_MIX_RETENTION): linear attention with one fixed decay g per head,
//   S_t = g S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t,
// q and k rotated, k over sqrt(d); the head's output is o / rms(o) silu(gate).  Everything is f32, products included (v_mfma_f32_16x16x4_f32); the state
// [group][H][dp][dvp] lives as long as its page group.
// Lightning attention (IXT_MIX_LIGHTNING): the same recurrence on silu(q), silu(k), silu(v) without a rotation and a factor, and one norm over all heads
// (join_norm): the outputs stay in memory until k_ret_join.
//
// Over a run of rows the recurrence goes by chunks of SEG_CHUNK rows (k_segments lists them).  Row i of a chunk (from 0), state S in front of it:
//   o_i = g^(i + 1) S^T q_i + sum_(j <= i) g^(i - j) (k_j . q_i) v_j,      S <- g^n S + sum_j g^(n - 1 - j) k_j v_j^T
//
//   k_ret_prep   projection slices -> rotated queries, rotated and scaled keys, values
//   k_ret_sums   chunk by chunk: U = sum_j g^(n - 1 - j) k_j v_j^T
//   k_ret_carry  run by run: the state in front of every chunk, in the place of its U; the group's new state
//   k_ret_out    chunk by chunk: the outputs (with up to 128 value dims also norm and gate; beyond: k_ret_gate)
//   k_ret_step   one token per row (decode): all of it in one launch (join_norm: up to the outputs)
//   k_ret_join   norm over all heads, weight, sigmoid gate
//
// Matrix products: lane (i = lane & 15, q = lane >> 4) holds element i of four terms 4 q + e of a 16-term step, e = 0 .. 3 being four instructions; the
// order of the terms is the same for both operands.  D: lane holds rows 4 q + e of column i.
#pragma once
#include "ixt_heads_kernels.h"

struct RetGeom {
  int H, d, dv, dp, dvp, rot;               // heads, key / value dims and both padded to 16, rotated dims
  int hs, vs, ok, ov, og;                   // projection columns: a query / key head takes hs, a value head (and its gate) vs
  int silu, join_norm;                      // silu on q, k, v; all heads normed together
  float kf;                                 // factor on the keys
  int oc, kend;                             // act of the output projection: the heads' first column, and where the zeros behind them end
  float of;                                 // factor on the outputs
};
__device__ __forceinline__ void ret_act4(const RetGeom& g, float f, const float* v, float* o) {
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = (g.silu ? v[j] * f32_sigmoid(v[j]) : v[j]) * f;
}
// pow [H][SEG_CHUNK + 1]: powers of a head's decay
struct RetArgs {
  RetGeom g; Slices t;
  const float* pow;
  const int32_t* seg; const int4* chunk; const int32_t* nseg;      // nseg[0] runs, nseg[1] chunks
  float *q, *k, *v;                         // [R][H][dp], [R][H][dp], [R][H][dvp]
  float *u, *state, *o;                     // [chunk][H][dp][dvp], [group][H][dp][dvp], [R][H][dvp]
  float eps;
};

// LP lanes per head: queries, keys, values.  grid (R, ceil(3 H LP / 256)), block 256.
template <int LP>
__global__ __launch_bounds__(256) void k_ret_prep(RetArgs a, HeadsRope rope, RowsArgs rows) {
  const RetGeom& g = a.g;
  const int r = blockIdx.x, j = blockIdx.y * (256 / LP) + threadIdx.x / LP, sl = threadIdx.x % LP;
  if (j >= 3 * g.H || !rows.active[r]) return;
  const int h = j % g.H, pos = rows.pos[r];
  if (j < 2 * g.H) {
    const bool key = j >= g.H;
    const float f = key ? g.kf : 1.0f;
    float* o = (key ? a.k : a.q) + ((size_t)r * g.H + h) * g.dp;
    head_norm_rotate<LP>(a.t, r, (key ? g.ok : 0) + h * g.hs, g, nullptr, 0.0f, rope, pos, g.dp, sl,
                         [&](int c, const float* v) { float u[4]; ret_act4(g, f, v, u); *reinterpret_cast<float4*>(o + c) = make_float4(u[0], u[1], u[2], u[3]); });
    return;
  }
  float* o = a.v + ((size_t)r * g.H + h) * g.dvp;
  for (int c = sl * 4; c < g.dvp; c += 4 * LP) {
    float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (c < g.vs) a.t.at4(r, g.ov + h * g.vs + c, v);
    ret_act4(g, 1.0f, v, v);
    *reinterpret_cast<float4*>(o + c) = make_float4(v[0], v[1], v[2], v[3]);
  }
}

// n (<= SEG_CHUNK) rows of W columns (from c0 on, as far as they exist) of x [row][heads][cols], times f(row) -> LDS [SEG_CHUNK][LD], zeros elsewhere
template <int W, int LD, typename F>
__device__ __forceinline__ void ret_stage(const float* __restrict__ x, int row0, int n, int H, int h, int cols, int c0, float* lds, int tid, F f) {
  constexpr int NIT = SEG_CHUNK * W / 1024;
  float4 v[NIT];
  float s[NIT];
#pragma unroll
  for (int it = 0; it < NIT; ++it) {                         // (everything requested before the first store)
    const int e = it * 256 + tid, j = e / (W / 4), c = e % (W / 4) * 4;
    v[it] = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (j < n && c0 + c < cols) v[it] = *reinterpret_cast<const float4*>(x + ((size_t)(row0 + j) * H + h) * cols + c0 + c);
    s[it] = f(j);
  }
#pragma unroll
  for (int it = 0; it < NIT; ++it) {
    const int e = it * 256 + tid, j = e / (W / 4), c = e % (W / 4) * 4;
    *reinterpret_cast<float4*>(lds + j * LD + c) = make_float4(v[it].x * s[it], v[it].y * s[it], v[it].z * s[it], v[it].w * s[it]);
  }
}

// U of a chunk: a block owns 64 x 128 of a head's [dp][dvp] (a wave 16 key rows).  grid (chunks, H, ceil(dp / 64) ceil(dvp / 128)), block 256.
static __global__ __launch_bounds__(256, 2) void k_ret_sums(RetArgs a) {
  constexpr int LDK = 64 + 16, LDV = 128 + 16;      // (four token rows side by side cover the banks once)
  __shared__ __attribute__((aligned(16))) float ks[SEG_CHUNK * LDK], vs[SEG_CHUNK * LDV];
  const RetGeom& g = a.g;
  const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i16 = lane & 15, q4 = lane >> 4;
  if (ch >= a.nseg[1]) return;
  const int4 c = a.chunk[ch];
  const int nv = (g.dvp + 127) / 128, d0 = blockIdx.z / nv * 64, v0 = blockIdx.z % nv * 128, n = c.y;
  const float* pw = a.pow + h * (SEG_CHUNK + 1);
  ret_stage<64, LDK>(a.k, c.x, n, g.H, h, g.dp, d0, ks, tid, [&](int j) { return pw[max(n - 1 - j, 0)]; });
  ret_stage<128, LDV>(a.v, c.x, n, g.H, h, g.dvp, v0, vs, tid, [](int) { return 1.0f; });
  __syncthreads();
  const int dr = d0 + wave * 16;
  if (dr >= g.dp) return;
  f32x4 acc[8];
#pragma unroll
  for (int t = 0; t < 8; ++t) acc[t] = f32x4(0.0f);
  const int steps = (n + 3) / 4;
  for (int s = 0; s < steps; ++s) {
    const int j = s * 4 + q4;
    const float kf = ks[j * LDK + wave * 16 + i16];
#pragma unroll
    for (int t = 0; t < 8; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(vs[j * LDV + t * 16 + i16], kf, acc[t], 0, 0, 0);      // D[value][key row]
  }
  float* u = a.u + (((size_t)ch * g.H + h) * g.dp + dr + i16) * g.dvp + v0 + q4 * 4;
#pragma unroll
  for (int t = 0; t < 8; ++t)
    if (v0 + t * 16 < g.dvp) *reinterpret_cast<float4*>(u + t * 16) = make_float4(acc[t][0], acc[t][1], acc[t][2], acc[t][3]);
}

// grid (runs, H, ceil(dp dvp / 1024)), block 256: four elements of the state per thread, the chunks of a run one after the other (the next ones' U on their way)
static __global__ __launch_bounds__(256) void k_ret_carry(RetArgs a) {
  const RetGeom& g = a.g;
  const int s = blockIdx.x, h = blockIdx.y;
  if (s >= a.nseg[0]) return;
  const int n = a.seg[s * 8 + 1], grp = a.seg[s * 8 + 2], start = a.seg[s * 8 + 3], base = a.seg[s * 8 + 5];
  const size_t per = (size_t)g.dp * g.dvp, e = ((size_t)blockIdx.z * 256 + threadIdx.x) * 4;
  if (n <= 0 || e >= per) return;
  const float* pw = a.pow + h * (SEG_CHUNK + 1);
  float4* sp = reinterpret_cast<float4*>(a.state + ((size_t)grp * g.H + h) * per + e);
  float4 S = start > 0 ? *sp : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  const int nc = (n + SEG_CHUNK - 1) / SEG_CHUNK;
  const size_t step = (size_t)g.H * per;
  float* u = a.u + ((size_t)base * g.H + h) * per + e;
  constexpr int A = 4;                                       // chunks in flight
  float4 nx[A];
#pragma unroll
  for (int i = 0; i < A; ++i) nx[i] = *reinterpret_cast<const float4*>(u + min(i, nc - 1) * step);
  for (int c0 = 0; c0 < nc; c0 += A) {
    float4 cu[A];
#pragma unroll
    for (int i = 0; i < A; ++i) cu[i] = nx[i];
    if (c0 + A < nc) {
#pragma unroll
      for (int i = 0; i < A; ++i) nx[i] = *reinterpret_cast<const float4*>(u + min(c0 + A + i, nc - 1) * step);
    }
#pragma unroll
    for (int i = 0; i < A; ++i) {
      if (c0 + i >= nc) break;
      const float f = pw[min(SEG_CHUNK, n - (c0 + i) * SEG_CHUNK)];
      *reinterpret_cast<float4*>(u + (c0 + i) * step) = S;
      S = make_float4(fmaf(f, S.x, cu[i].x), fmaf(f, S.y, cu[i].y), fmaf(f, S.z, cu[i].z), fmaf(f, S.w, cu[i].w));
    }
  }
  *sp = S;
}

// four columns of a head's output, normed by rs, times silu of their gates and the layer's factor
__device__ __forceinline__ void ret_gate4(const Slices& t, int r, const RetGeom& g, int h, int c, float rs, float* v) {
  rs *= g.of;
  float z[4];
  t.at4(r, g.og + h * g.vs + c, z);
#pragma unroll
  for (int j = 0; j < 4; ++j) v[j] *= rs * z[j] * f32_sigmoid(z[j]);
}

// Outputs: a block owns up to 16 NT value columns of a (chunk, head), a wave 16 rows.  First P^T = K Q^T (its lanes hold the operand of the product with the
// values), then S^T Q^T times g^(i + 1), then V^T P^T.  Keys, then the state, pass through one LDS buffer 64 key dims at a time.
// FUSED: all value dims are here; norm and gate follow on chip.  grid (chunks, H, ceil(dvp / (16 NT))), block 256.
template <typename T, int NT, bool FUSED>
__global__ __launch_bounds__(256, 2) void k_ret_out(RetArgs a, T* __restrict__ out, int Kp) {
  constexpr int W = NT * 16, LDK = 64 + 4, LDV = W + 4, KS = SEG_CHUNK * (LDK > LDV ? LDK : LDV);      // (every fourth row: 16 banks on)
  __shared__ __attribute__((aligned(16))) float ks[KS], vs[SEG_CHUNK * LDV];
  const RetGeom& g = a.g;
  const int ch = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * W, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, i16 = lane & 15, q4 = lane >> 4;
  if (ch >= a.nseg[1]) return;
  const int4 c = a.chunk[ch];
  const int n = c.y, row = c.x + wave * 16 + i16;
  const bool ok = wave * 16 + i16 < n, first = c.w == 0 && a.seg[c.z * 8 + 3] == 0;      // first: nothing stands in the state yet
  const float* pw = a.pow + h * (SEG_CHUNK + 1);
  const float* qp = a.q + ((size_t)(ok ? row : c.x) * g.H + h) * g.dp;
  ret_stage<W, LDV>(a.v, c.x, n, g.H, h, g.dvp, v0, vs, tid, [](int) { return 1.0f; });
  f32x4 p[4];
#pragma unroll
  for (int t = 0; t < 4; ++t) p[t] = f32x4(0.0f);
  for (int d0 = 0; d0 < g.dp; d0 += 64) {
    const int steps = min(4, (g.dp - d0) / 16);
    f32x4 q[4];                                              // (on their way together with the keys)
#pragma unroll
    for (int s = 0; s < 4; ++s) q[s] = *reinterpret_cast<const f32x4*>(qp + d0 + min(s, steps - 1) * 16 + q4 * 4);
    if (d0 > 0) __syncthreads();
    ret_stage<64, LDK>(a.k, c.x, n, g.H, h, g.dp, d0, ks, tid, [](int) { return 1.0f; });
    __syncthreads();
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      if (s >= steps) continue;
      const f32x4 qf = q[s];
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        if (t > wave) continue;                              // keys behind the wave's rows
        const f32x4 kf = *reinterpret_cast<const f32x4*>(ks + (t * 16 + i16) * LDK + s * 16 + q4 * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) p[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[e], qf[e], p[t], 0, 0, 0);      // D[key][row]
      }
    }
  }
  f32x4 o[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) o[t] = f32x4(0.0f);
  if (!first) {
    const float* sp = a.u + ((size_t)ch * g.H + h) * g.dp * g.dvp;
    for (int d0 = 0; d0 < g.dp; d0 += 64) {
      const int steps = min(4, (g.dp - d0) / 16);
      f32x4 q[4];
#pragma unroll
      for (int s = 0; s < 4; ++s) q[s] = *reinterpret_cast<const f32x4*>(qp + d0 + min(s, steps - 1) * 16 + q4 * 4);
      float4 sv[SEG_CHUNK * W / 1024];                       // 64 key rows of the state, requested while the buffer is still being read
#pragma unroll
      for (int it = 0; it < SEG_CHUNK * W / 1024; ++it) {
        const int e = it * 256 + tid, j = e / (W / 4), cc = e % (W / 4) * 4;
        sv[it] = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
        if (d0 + j < g.dp && v0 + cc < g.dvp) sv[it] = *reinterpret_cast<const float4*>(sp + (size_t)(d0 + j) * g.dvp + v0 + cc);
      }
      __syncthreads();
#pragma unroll
      for (int it = 0; it < SEG_CHUNK * W / 1024; ++it) {
        const int e = it * 256 + tid, j = e / (W / 4), cc = e % (W / 4) * 4;
        *reinterpret_cast<float4*>(ks + j * LDV + cc) = sv[it];
      }
      __syncthreads();
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        if (s >= steps) continue;
        const f32x4 qf = q[s];
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
          for (int t = 0; t < NT; ++t) o[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(ks[(s * 16 + q4 * 4 + e) * LDV + t * 16 + i16], qf[e], o[t], 0, 0, 0);      // D[value][row]
      }
    }
    const float f = pw[min(wave * 16 + i16 + 1, SEG_CHUNK)];
#pragma unroll
    for (int t = 0; t < NT; ++t) o[t] = o[t] * f;
  }
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    if (t > wave) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int back = (wave - t) * 16 + i16 - (q4 * 4 + e);      // row - key
      const float w = back >= 0 ? p[t][e] * pw[back] : 0.0f;
#pragma unroll
      for (int u = 0; u < NT; ++u) o[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(vs[(t * 16 + q4 * 4 + e) * LDV + u * 16 + i16], w, o[u], 0, 0, 0);
    }
  }
  if constexpr (FUSED) {
    float ss = 0.0f;
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(o[t][e], o[t][e], ss);
    ss += __shfl_xor(ss, 16, 64);
    ss += __shfl_xor(ss, 32, 64);
    if (!ok) return;
    const float rs = 1.0f / sqrtf(ss / (float)g.dv + a.eps);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int cc = t * 16 + q4 * 4;
      if (cc >= g.vs) continue;
      float v[4] = {o[t][0], o[t][1], o[t][2], o[t][3]};
      ret_gate4(a.t, row, g, h, cc, rs, v);
      act_store4(out, row, g.oc + h * g.vs + cc, Kp, v);
    }
    const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (h == g.H - 1)
      for (int k = g.oc + g.H * g.vs + q4 * 4; k < g.kend; k += 16) act_store4(out, row, k, Kp, z);
  } else {
    if (!ok) return;
#pragma unroll
    for (int t = 0; t < NT; ++t)
      if (v0 + t * 16 < g.dvp) *reinterpret_cast<float4*>(a.o + ((size_t)row * g.H + h) * g.dvp + v0 + t * 16 + q4 * 4) = make_float4(o[t][0], o[t][1], o[t][2], o[t][3]);
  }
}
// norm and gate of outputs in memory.  grid (R, ceil(H / 4)), block 256: a wave per head.
template <typename T>
__global__ __launch_bounds__(256) void k_ret_gate(RetArgs a, const int32_t* __restrict__ row_active, T* __restrict__ out, int Kp) {
  const RetGeom& g = a.g;
  const int r = blockIdx.x, h = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (h >= g.H || !row_active[r]) return;
  const float* oh = a.o + ((size_t)r * g.H + h) * g.dvp;
  float ss = 0.0f;
  for (int c = lane; c < g.dv; c += 64) ss = fmaf(oh[c], oh[c], ss);
  const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)g.dv + a.eps);
  for (int c = lane * 4; c < g.vs; c += 256) {
    const float4 u = *reinterpret_cast<const float4*>(oh + c);
    float v[4] = {u.x, u.y, u.z, u.w};
    ret_gate4(a.t, r, g, h, c, rs, v);
    act_store4(out, r, g.oc + h * g.vs + c, Kp, v);
  }
  const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  if (h == g.H - 1)
    for (int k = g.oc + g.H * g.vs + lane * 4; k < g.kend; k += 256) act_store4(out, r, k, Kp, z);
}
// all heads of a row: o / rms(o) w sigmoid(gate); w [H][vs], zeros behind a head's dv.  A block of 256.
template <typename T>
__device__ __forceinline__ void ret_join(const RetArgs& a, const float* __restrict__ w, const int32_t* __restrict__ row_active, T* __restrict__ out, int Kp, const int r) {
  __shared__ float red[4];
  const RetGeom& g = a.g;
  const int tid = threadIdx.x, n = g.H * g.vs;
  if (!row_active[r]) return;
  const float* o = a.o + (size_t)r * g.H * g.dvp;
  constexpr int B = 4;                                       // columns of a thread that stay in registers, in fours
  float4 v[B], z[B];
  float ss = 0.0f;
#pragma unroll
  for (int i = 0; i < B; ++i) {
    const int c = (i * 256 + tid) * 4;
    v[i] = z[i] = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (c < n) {
      v[i] = *reinterpret_cast<const float4*>(o + c / g.vs * g.dvp + c % g.vs);      // (columns from dv on are zero)
      a.t.at4(r, g.og + c, &z[i].x);
    }
  }
#pragma unroll
  for (int i = 0; i < B; ++i) ss = fmaf(v[i].x, v[i].x, fmaf(v[i].y, v[i].y, fmaf(v[i].z, v[i].z, fmaf(v[i].w, v[i].w, ss))));
  for (int c = (B * 256 + tid) * 4; c < n; c += 1024) {
    const float4 u = *reinterpret_cast<const float4*>(o + c / g.vs * g.dvp + c % g.vs);
    ss = fmaf(u.x, u.x, fmaf(u.y, u.y, fmaf(u.z, u.z, fmaf(u.w, u.w, ss))));
  }
  const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)(g.H * g.dv) + a.eps) * g.of;
  auto put = [&](int c, const float4& u, const float4& y) {
    const float4 ww = *reinterpret_cast<const float4*>(w + c);
    const float q[4] = {u.x * rs * ww.x * f32_sigmoid(y.x), u.y * rs * ww.y * f32_sigmoid(y.y), u.z * rs * ww.z * f32_sigmoid(y.z), u.w * rs * ww.w * f32_sigmoid(y.w)};
    act_store4(out, r, g.oc + c, Kp, q);
  };
#pragma unroll
  for (int i = 0; i < B; ++i)
    if ((i * 256 + tid) * 4 < n) put((i * 256 + tid) * 4, v[i], z[i]);
  for (int c = (B * 256 + tid) * 4; c < n; c += 1024) {
    const float4 u = *reinterpret_cast<const float4*>(o + c / g.vs * g.dvp + c % g.vs);
    float4 y;
    a.t.at4(r, g.og + c, &y.x);
    put(c, u, y);
  }
  const float zero[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int k = g.oc + n + tid * 4; k < g.kend; k += 1024) act_store4(out, r, k, Kp, zero);
}
// grid R, block 256
template <typename T>
__global__ __launch_bounds__(256) void k_ret_join(RetArgs a, const float* __restrict__ w, const int32_t* __restrict__ row_active, T* __restrict__ out, int Kp) {
  ret_join<T>(a, w, row_active, out, Kp, blockIdx.x);
}

// Decode: block = (row, head).  A thread owns four value columns and every `ns`-th key row; the first of them are requested before anything else.
// A block of 256, LDS (2 dp + dvp + ns dvp) floats, ns = 256 / (dvp / 4).
template <typename T>
__device__ __forceinline__ void ret_step(const RetArgs& a, const HeadsRope& rope, const RowsArgs& rows, T* __restrict__ out, int Kp, const int r, const int h, float* sm) {
  __shared__ float red[4];
  const RetGeom& g = a.g;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int active = rows.active[r], pos = rows.pos[r], grp = rows.slot[r];      // (requested together)
  if (!active) return;
  float *qs = sm, *ks = sm + g.dp, *vs = ks + g.dp, *os = vs + g.dvp;
  const int ncg = g.dvp / 4, ns = 256 / ncg, sl = tid / ncg, cg = tid % ncg;
  const bool mine = sl < ns;
  float* sp = a.state + (((size_t)grp * g.H + h) * g.dp) * g.dvp + cg * 4;
  constexpr int B = 16;                                      // key rows in flight per thread
  float4 S[B];
#pragma unroll
  for (int i = 0; i < B; ++i) {
    const int d = sl + i * ns;
    S[i] = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (mine && pos > 0 && d < g.d) S[i] = *reinterpret_cast<const float4*>(sp + (size_t)d * g.dvp);
  }
  if (wave < 2) {
    const float f = wave == 1 ? g.kf : 1.0f;
    float* o = wave == 1 ? ks : qs;
    head_norm_rotate<64>(a.t, r, (wave == 1 ? g.ok : 0) + h * g.hs, g, nullptr, 0.0f, rope, pos, g.dp, lane,
                         [&](int c, const float* v) { float u[4]; ret_act4(g, f, v, u); *reinterpret_cast<float4*>(o + c) = make_float4(u[0], u[1], u[2], u[3]); });
  } else if (wave == 2) {
    for (int c = lane * 4; c < g.dvp; c += 256) {
      float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
      if (c < g.vs) a.t.at4(r, g.ov + h * g.vs + c, v);
      ret_act4(g, 1.0f, v, v);
      *reinterpret_cast<float4*>(vs + c) = make_float4(v[0], v[1], v[2], v[3]);
    }
  }
  const float decay = a.pow[h * (SEG_CHUNK + 1) + 1];
  __syncthreads();
  float4 acc = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  if (mine) {
    const float4 v = *reinterpret_cast<const float4*>(vs + cg * 4);
    for (int d0 = sl; d0 < g.d; d0 += B * ns) {
      if (d0 > sl) {
#pragma unroll
        for (int i = 0; i < B; ++i) {
          const int d = d0 + i * ns;
          if (pos > 0 && d < g.d) S[i] = *reinterpret_cast<const float4*>(sp + (size_t)d * g.dvp);
        }
      }
#pragma unroll
      for (int i = 0; i < B; ++i) {
        const int d = d0 + i * ns;
        if (d >= g.d) continue;
        const float kd = ks[d], qd = qs[d];
        const float4 n = make_float4(fmaf(decay, S[i].x, kd * v.x), fmaf(decay, S[i].y, kd * v.y), fmaf(decay, S[i].z, kd * v.z), fmaf(decay, S[i].w, kd * v.w));
        *reinterpret_cast<float4*>(sp + (size_t)d * g.dvp) = n;
        acc.x = fmaf(qd, n.x, acc.x); acc.y = fmaf(qd, n.y, acc.y); acc.z = fmaf(qd, n.z, acc.z); acc.w = fmaf(qd, n.w, acc.w);
      }
    }
    *reinterpret_cast<float4*>(os + sl * g.dvp + cg * 4) = acc;
  }
  __syncthreads();
  float4 o = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  if (tid < ncg)
    for (int s = 0; s < ns; ++s) {
      const float4 p = *reinterpret_cast<const float4*>(os + s * g.dvp + tid * 4);
      o.x += p.x; o.y += p.y; o.z += p.z; o.w += p.w;
    }
  if (g.join_norm) {
    if (tid < ncg) *reinterpret_cast<float4*>(a.o + ((size_t)r * g.H + h) * g.dvp + tid * 4) = o;
    return;
  }
  const float ss = fmaf(o.x, o.x, fmaf(o.y, o.y, fmaf(o.z, o.z, o.w * o.w)));      // (columns from dv on are zero)
  const float rs = 1.0f / sqrtf(block_sum256(ss, red) / (float)g.dv + a.eps);
  if (tid * 4 < g.vs) {
    float v[4] = {o.x, o.y, o.z, o.w};
    ret_gate4(a.t, r, g, h, tid * 4, rs, v);
    act_store4(out, r, g.oc + h * g.vs + tid * 4, Kp, v);
  }
  const float z[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  if (h == g.H - 1)
    for (int k = g.oc + g.H * g.vs + tid * 4; k < g.kend; k += 1024) act_store4(out, r, k, Kp, z);
}
// grid (R, H), block 256
template <typename T>
__global__ __launch_bounds__(256) void k_ret_step(RetArgs a, HeadsRope rope, RowsArgs rows, T* __restrict__ out, int Kp) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  ret_step<T>(a, rope, rows, out, Kp, blockIdx.x, blockIdx.y, sm);
}

// Attention over heads and a retention side by side, one token per row: the blocks of both in one launch, which is as long as the longer of the two and not
// as their sum.  grid R H + R G hchunks nsplit, block 256, LDS the larger of the two.
template <int DK, int DV>
__global__ __launch_bounds__(256, 2) void k_pair_decode(HeadsAttnArgs a, int nsplit, RetArgs b, HeadsRope rope, int Kp) {
  extern __shared__ __attribute__((aligned(16))) bf16_t tile[];
  int i = blockIdx.x;
  if (i < a.R * b.g.H) { ret_step<bf16_t>(b, rope, a.rows, a.out, Kp, i / b.g.H, i % b.g.H, reinterpret_cast<float*>(tile)); return; }
  i -= a.R * b.g.H;
  const int hb = a.g.G * a.hchunks;
  heads_decode<DK, DV, true, 1>(a, i / nsplit / hb, i / nsplit % hb, i % nsplit, nsplit, tile);
}
// their second half: key splits put together, the retention's heads normed together.  grid (R, H + 1), block 256.
static __global__ __launch_bounds__(256) void k_pair_join(HeadsAttnArgs a, int nsplit, RetArgs b, const float* __restrict__ w, int Kp) {
  if ((int)blockIdx.y < a.g.H) heads_combine(a.part_o, a.part_ml, nsplit, a.g, a.mp, a.t, a.rows.active, a.out, Kp, blockIdx.x, blockIdx.y);
  else ret_join<bf16_t>(b, w, a.rows.active, a.out, Kp, blockIdx.x);
}
