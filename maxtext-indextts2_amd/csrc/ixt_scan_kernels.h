// ixt_scan_kernels.h -- selective scan (IXT_MIX_SCAN): per channel c and state n
//   S <- exp(dt_c A[c, n]) S + dt_c x_c B_n,   y_c = sum_n S[c, n] C_n + D_c x_c,   output y silu(z),
// dt = softplus(projection + bias), A = -exp(A_log); x behind a short causal convolution with bias and silu.  Everything from dt on is f32; the state
// [group][C][Np] lives as long as its page group.
//
// Over a run of rows the recurrence goes by chunks of SEG_CHUNK rows (k_segments lists them): the state behind a chunk is exp(A sum dt) times the one in
// front of it plus what the chunk leaves by itself.
//
//   k_scan_conv   projection slices -> x, the operand of the next projection, where every later kernel reads it and the outputs take its place
//   k_scan_rank   the step-size part of that projection as the operand of the third one
//   k_scan_sums   chunk by chunk: U = the state a chunk leaves from zero, and its sum of dt; the step sizes in the place of their projection
//   k_scan_carry  run by run: the state in front of every chunk, in the place of its U; the group's new state
//   k_scan_out    chunk by chunk: the outputs
//   k_scan_step   one token per row (decode)
//
// A channel's states lie on LPC = Np / SPL neighbouring lanes, SPL each.
#pragma once
#include "ixt_hybrid_kernels.h"

struct ScanGeom {
  int C, Cp, N, Np, rank, taps;             // channels, padded to 4; states, padded to a power of two from 16 on; rank of the step sizes, convolution taps
  int oz, ob, oc;                           // columns: z in the input projection; B and C in the second one
};
struct ScanArgs {
  ScanGeom g; Slices in, low, dt;           // the three projections (dt: the third one, with its bias)
  float* dts;                               // the first slice of dt
  const float *a2, *D;                      // [C][Np]: -exp(A_log) log2(e), zeros behind N; [Cp]
  const int32_t* seg; const int4* chunk; const int32_t* nseg;
  float *u, *sum, *state;                   // [chunk][C][Np], [chunk][Cp], [group][C][Np]
};

// a2 in place from A_log.  Padding stays zero.
static __global__ __launch_bounds__(256) void k_scan_rates(float* __restrict__ a2, int C, int N, int Np) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < C * Np && i % Np < N) a2[i] = -1.44269504088896340736f * expf(a2[i]);
}

// four elements of an operand (k0 % 4 == 0)
__device__ __forceinline__ float4 act_load4(const bf16_t* b, int r, int k0, int Kp) {
  const uint2 v = *reinterpret_cast<const uint2*>(b + xidx(r, k0, Kp));
  return make_float4(bflo(v.x), bfhi(v.x), bflo(v.y), bfhi(v.y));
}
__device__ __forceinline__ float4 act_load4(const float* b, int r, int k0, int Kp) { return *reinterpret_cast<const float4*>(b + (size_t)r * Kp + k0); }

// Convolution, bias, silu.  Weights [taps][Cp], tails [group][2][taps - 1][Cp].  grid (ceil(R / RB), ceil(Kp / 1024)), block 256: four channels of RB rows per
// thread; rows in the middle of a run (taps 4, one slice) share their inputs.
struct ScanConvArgs {
  Slices t; ScanGeom g; const float *w, *bias; const int32_t *row_seg, *row_j, *seg;
  float* tails; int R;
};
__device__ __forceinline__ void fma4(const float4& x, const float4& w, float* v) { v[0] = fmaf(x.x, w.x, v[0]); v[1] = fmaf(x.y, w.y, v[1]); v[2] = fmaf(x.z, w.z, v[2]); v[3] = fmaf(x.w, w.w, v[3]); }
// one row, any place in its run, any number of taps: v from the bias to the convolution; leaves what the next run needs
__device__ __forceinline__ void scan_conv_row(const ScanConvArgs& a, int r, int s, int c, float* v) {
  const ScanGeom& g = a.g;
  const int32_t* sg = a.seg + (size_t)s * 8;
  const int n = sg[1], start = sg[3], par = sg[4], j = a.row_j[r], taps = g.taps;
  const size_t tsz = (size_t)(taps - 1) * g.Cp;
  const float* tin = a.tails + ((size_t)sg[2] * 2 + par) * tsz + c;
  float* tout = a.tails + ((size_t)sg[2] * 2 + (par ^ 1)) * tsz + c;
  float x0[4];
  a.t.at4(r, c, x0);
  const float4 here = make_float4(x0[0], x0[1], x0[2], x0[3]);
  fma4(here, *reinterpret_cast<const float4*>(a.w + (size_t)(taps - 1) * g.Cp + c), v);
  for (int b0 = 1; b0 < taps; b0 += 3) {                     // three earlier inputs in flight: rows of the run, or what is kept of those before it (oldest first)
    float4 x[3], w[3];
#pragma unroll
    for (int i = 0; i < 3; ++i) {
      const int back = min(b0 + i, taps - 1);
      const bool mine = j - back >= 0;
      const float* src = mine ? a.t.p + (size_t)(r - back) * a.t.ncols + c : tin + (size_t)max(taps - 1 - (back - j), 0) * g.Cp;
      x[i] = mine || start > 0 ? *reinterpret_cast<const float4*>(src) : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
      w[i] = b0 + i < taps ? *reinterpret_cast<const float4*>(a.w + (size_t)(taps - 1 - back) * g.Cp + c) : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
      if (mine)
        for (int q = 1; q < a.t.n; ++q) {
          const float4 u = *reinterpret_cast<const float4*>(src + (size_t)q * a.t.stride);
          x[i].x += u.x; x[i].y += u.y; x[i].z += u.z; x[i].w += u.w;
        }
    }
#pragma unroll
    for (int i = 0; i < 3; ++i) fma4(x[i], w[i], v);
  }
  const int dist = n - 1 - j;                                // the last taps - 1 inputs stay
  if (dist < taps - 1) *reinterpret_cast<float4*>(tout + (size_t)(taps - 2 - dist) * g.Cp) = here;
  if (dist == 0)
    for (int e = n; e < taps - 1; ++e)
      *reinterpret_cast<float4*>(tout + (size_t)(taps - 2 - e) * g.Cp) = start > 0 ? *reinterpret_cast<const float4*>(tin + (size_t)(taps - 2 - (e - n)) * g.Cp) : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
}
template <typename T, int RB>
__global__ __launch_bounds__(256) void k_scan_conv(ScanConvArgs a, T* __restrict__ out, int Kp) {
  const ScanGeom& g = a.g;
  const int r0 = blockIdx.x * RB, c = (blockIdx.y * 256 + threadIdx.x) * 4, nr = min(RB, a.R - r0);
  if (c >= Kp) return;
  float4 b = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  const bool real = c < g.Cp;                                // (everything is zero in channels C .. Cp - 1, and there is nothing from Cp on)
  if (real) b = *reinterpret_cast<const float4*>(a.bias + c);
  auto put = [&](int r, float* v) {
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] *= f32_sigmoid(v[e]);
    act_store4(out, r, c, Kp, v);
  };
  if constexpr (RB > 1) {
    const int s = a.row_seg[r0], j = a.row_j[r0];
    if (nr == RB && real && g.taps == 4 && a.t.n == 1 && a.t.bias == nullptr && s >= 0 && j >= 3 && a.row_seg[r0 + RB - 1] == s && j + RB - 1 + 3 < a.seg[(size_t)s * 8 + 1]) {
      float4 x[RB + 3], w[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) w[i] = *reinterpret_cast<const float4*>(a.w + (size_t)i * g.Cp + c);
#pragma unroll
      for (int i = 0; i < RB + 3; ++i) x[i] = *reinterpret_cast<const float4*>(a.t.p + (size_t)(r0 + i - 3) * a.t.ncols + c);
#pragma unroll
      for (int i = 0; i < RB; ++i) {
        float v[4] = {b.x, b.y, b.z, b.w};
        fma4(x[i + 3], w[3], v); fma4(x[i + 2], w[2], v); fma4(x[i + 1], w[1], v); fma4(x[i], w[0], v);      // (the order of scan_conv_row)
        put(r0 + i, v);
      }
      return;
    }
  }
  for (int i = 0; i < nr; ++i) {
    const int r = r0 + i, s = a.row_seg[r];
    if (s < 0) continue;
    float v[4] = {b.x, b.y, b.z, b.w};
    if (real) scan_conv_row(a, r, s, c, v);
    put(r, v);
  }
}

// The second projection's slices are added up in the first one, too.  grid (R), block 64: four columns per thread and round.  first: the first slice
template <typename T>
__global__ __launch_bounds__(64) void k_scan_rank(Slices low, float* __restrict__ first, int rank, T* __restrict__ out, int Kp) {
  const int r = blockIdx.x;
  for (int k = threadIdx.x * 4; k < max(Kp, low.n > 1 ? low.ncols : 0); k += 256) {
    float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (k < low.ncols) low.template at4<8>(r, k, v);
    if (k < low.ncols && low.n > 1) *reinterpret_cast<float4*>(first + (size_t)r * low.ncols + k) = make_float4(v[0], v[1], v[2], v[3]);
    if (k >= Kp) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (k + e >= rank) v[e] = 0.0f;
    act_store4(out, r, k, Kp, v);
  }
}

// sum over the LPC (1, 2, 4, .. 64) lanes of a channel, every lane ends up with it
template <int LPC>
__device__ __forceinline__ float lanes_sum(float v) {
  if constexpr (LPC > 1) v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xf, 0xf, false));      // quad_perm 1 0 3 2
  if constexpr (LPC > 2) v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xf, 0xf, false));      // quad_perm 2 3 0 1
#pragma unroll
  for (int off = 4; off < LPC; off <<= 1) v += __shfl_xor(v, off, 64);
  return v;
}

// the value of lane i (0 .. 3, a constant) of this lane's four
__device__ __forceinline__ float quad_lane(float v, int i) {
  const int x = __float_as_int(v);
  return __int_as_float(i == 0 ? __builtin_amdgcn_update_dpp(0, x, 0x00, 0xf, 0xf, false) : i == 1 ? __builtin_amdgcn_update_dpp(0, x, 0x55, 0xf, 0xf, false)
                        : i == 2 ? __builtin_amdgcn_update_dpp(0, x, 0xAA, 0xf, 0xf, false) : __builtin_amdgcn_update_dpp(0, x, 0xFF, 0xf, 0xf, false));
}

// A chunk's operands -> LDS: {dt, dt x} [SEG_CHUNK][CB] of CB channels from c0 on, the B (and C) columns [SEG_CHUNK][Np]; zeros behind the chunk's rows: such
// a token changes nothing.  OUT: the step sizes are in place already (k_scan_sums)
template <typename T, int SPL, int LPC, bool OUT>
__device__ __forceinline__ void scan_stage(const ScanArgs& a, const int4& c, int c0, const T* __restrict__ act, int Kp, float2* ds, float* bs, float* cs) {
  constexpr int CB = 256 / LPC, NP = SPL * LPC, QB = CB / 4, QN = NP / 4;
  const ScanGeom& g = a.g;
  const int tid = threadIdx.x, n = c.y;
#pragma unroll 4
  for (int i = tid; i < SEG_CHUNK * QB; i += 256) {
    const int j = i / QB, q = i % QB * 4, ch = c0 + q;
    float d[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    float4 x = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (j < n && ch < g.Cp) {                                // (in columns C .. Cp - 1 x is zero)
      x = act_load4(act, c.x + j, ch, Kp);
      if (OUT) {
        const float4 u = *reinterpret_cast<const float4*>(a.dts + (size_t)(c.x + j) * a.dt.ncols + ch);
        d[0] = u.x; d[1] = u.y; d[2] = u.z; d[3] = u.w;
      } else {
        a.dt.at4(c.x + j, ch, d);
#pragma unroll
        for (int e = 0; e < 4; ++e) d[e] = hw_softplus(d[e]);
        *reinterpret_cast<float4*>(a.dts + (size_t)(c.x + j) * a.dt.ncols + ch) = make_float4(d[0], d[1], d[2], d[3]);
      }
    }
    float4* o = reinterpret_cast<float4*>(ds + j * CB + q);
    o[0] = make_float4(d[0], d[0] * x.x, d[1], d[1] * x.y);
    o[1] = make_float4(d[2], d[2] * x.z, d[3], d[3] * x.w);
  }
  for (int i = tid; i < SEG_CHUNK * QN; i += 256) {
    const int j = i / QN, q = i % QN * 4;
    float b[4] = {0.0f, 0.0f, 0.0f, 0.0f}, y[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (j < n && q < g.N) {                                  // (columns behind N are zero up to the next multiple of 16)
      a.low.at4(c.x + j, g.ob + q, b);
      if (OUT) a.low.at4(c.x + j, g.oc + q, y);
    }
    *reinterpret_cast<float4*>(bs + j * NP + q) = make_float4(b[0], b[1], b[2], b[3]);
    if (OUT) *reinterpret_cast<float4*>(cs + j * NP + q) = make_float4(y[0], y[1], y[2], y[3]);
  }
}
template <int SPL, int LPC, bool OUT> constexpr size_t scan_lds() { return sizeof(float) * SEG_CHUNK * (2 * (256 / LPC) + (OUT ? 2 : 1) * SPL * LPC); }
template <int N>
__device__ __forceinline__ void lds_read(const float* p, float* v) {      // N a multiple of 4
#pragma unroll
  for (int i = 0; i < N; i += 4) { const float4 u = *reinterpret_cast<const float4*>(p + i); v[i] = u.x; v[i + 1] = u.y; v[i + 2] = u.z; v[i + 3] = u.w; }
}

// grid (chunks, ceil(C / CB)), block 256, LDS scan_lds<SPL, LPC, false>()
template <typename T, int SPL, int LPC>
__global__ __launch_bounds__(256) void k_scan_sums(ScanArgs a, const T* __restrict__ act, int Kp) {
  constexpr int CB = 256 / LPC, NP = SPL * LPC;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const ScanGeom& g = a.g;
  const int ch = blockIdx.x, tid = threadIdx.x, cl = tid / LPC, sub = tid % LPC, c0 = blockIdx.y * CB, col = c0 + cl;
  if (ch >= a.nseg[1]) return;
  const int4 c = a.chunk[ch];
  float2* ds = reinterpret_cast<float2*>(sm);
  float* bs = sm + 2 * SEG_CHUNK * CB;
  float a2[SPL], S[SPL];
  const size_t at = (size_t)min(col, g.C - 1) * NP + sub * SPL;
#pragma unroll
  for (int i = 0; i < SPL; ++i) { a2[i] = a.a2[at + i]; S[i] = 0.0f; }
  scan_stage<T, SPL, LPC, false>(a, c, c0, act, Kp, ds, bs, nullptr);
  __syncthreads();
  float sum = 0.0f;
  for (int j0 = 0; j0 < c.y; j0 += 4) {                      // (tokens behind the chunk's change nothing)
    float2 d[4];
    float b[4][SPL];
#pragma unroll
    for (int k = 0; k < 4; ++k) { d[k] = ds[(j0 + k) * CB + cl]; lds_read<SPL>(bs + (j0 + k) * NP + sub * SPL, b[k]); }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      sum += d[k].x;
#pragma unroll
      for (int i = 0; i < SPL; ++i) S[i] = fmaf(hw_exp2(d[k].x * a2[i]), S[i], d[k].y * b[k][i]);
    }
  }
  if (col >= g.C) return;
  float* u = a.u + (size_t)ch * g.C * NP + at;
#pragma unroll
  for (int i = 0; i < SPL; i += 4) *reinterpret_cast<float4*>(u + i) = make_float4(S[i], S[i + 1], S[i + 2], S[i + 3]);
  if (sub == 0) a.sum[(size_t)ch * g.Cp + col] = sum;
}

// grid (runs, ceil(C Np / 1024)), block 256: four states of a channel per thread, the chunks of a run one after the other (the next ones' U on their way)
static __global__ __launch_bounds__(256) void k_scan_carry(ScanArgs a) {
  const ScanGeom& g = a.g;
  const int s = blockIdx.x;
  if (s >= a.nseg[0]) return;
  const int n = a.seg[s * 8 + 1], grp = a.seg[s * 8 + 2], start = a.seg[s * 8 + 3], base = a.seg[s * 8 + 5];
  const size_t per = (size_t)g.C * g.Np, e = ((size_t)blockIdx.y * 256 + threadIdx.x) * 4;
  if (n <= 0 || e >= per) return;
  const float4 a2 = *reinterpret_cast<const float4*>(a.a2 + e);
  float4* sp = reinterpret_cast<float4*>(a.state + (size_t)grp * per + e);
  float4 S = start > 0 ? *sp : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  const int nc = (n + SEG_CHUNK - 1) / SEG_CHUNK;
  float* u = a.u + (size_t)base * per + e;
  const float* sum = a.sum + (size_t)base * g.Cp + e / g.Np;
  constexpr int A = 4;                                       // chunks in flight
  float4 nx[A];
  float ns[A];
#pragma unroll
  for (int i = 0; i < A; ++i) { nx[i] = *reinterpret_cast<const float4*>(u + min(i, nc - 1) * per); ns[i] = sum[(size_t)min(i, nc - 1) * g.Cp]; }
  for (int c0 = 0; c0 < nc; c0 += A) {
    float4 cu[A];
    float cs[A];
#pragma unroll
    for (int i = 0; i < A; ++i) { cu[i] = nx[i]; cs[i] = ns[i]; }
    if (c0 + A < nc) {
#pragma unroll
      for (int i = 0; i < A; ++i) { const size_t k = min(c0 + A + i, nc - 1); nx[i] = *reinterpret_cast<const float4*>(u + k * per); ns[i] = sum[k * g.Cp]; }
    }
#pragma unroll
    for (int i = 0; i < A; ++i) {
      if (c0 + i >= nc) break;
      *reinterpret_cast<float4*>(u + (c0 + i) * per) = S;
      S = make_float4(fmaf(hw_exp2(cs[i] * a2.x), S.x, cu[i].x), fmaf(hw_exp2(cs[i] * a2.y), S.y, cu[i].y), fmaf(hw_exp2(cs[i] * a2.z), S.z, cu[i].z),
                      fmaf(hw_exp2(cs[i] * a2.w), S.w, cu[i].w));
    }
  }
  *sp = S;
}

// the output of four channels: (y + D x) silu(z), in the place of x
template <typename T>
__device__ __forceinline__ void scan_put4(const ScanArgs& a, int r, int c, const float* y, T* act, int Kp) {
  const float4 x = act_load4(act, r, c, Kp), D = *reinterpret_cast<const float4*>(a.D + c);
  float z[4], v[4];
  a.in.at4(r, a.g.oz + c, z);                                // (z is zero in channels C .. Cp - 1)
  v[0] = fmaf(D.x, x.x, y[0]); v[1] = fmaf(D.y, x.y, y[1]); v[2] = fmaf(D.z, x.z, y[2]); v[3] = fmaf(D.w, x.w, y[3]);
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] *= z[e] * f32_sigmoid(z[e]);
  act_store4(act, r, c, Kp, v);
}

// grid (chunks, ceil(C / CB)), block 256, LDS scan_lds<SPL, LPC, true>()
template <typename T, int SPL, int LPC>
__global__ __launch_bounds__(256) void k_scan_out(ScanArgs a, T* __restrict__ act, int Kp) {
  constexpr int CB = 256 / LPC, NP = SPL * LPC, QB = CB / 4, TT = SPL > 8 ? 2 : 4;      // tokens whose operands are read together
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const ScanGeom& g = a.g;
  const int ch = blockIdx.x, tid = threadIdx.x, cl = tid / LPC, sub = tid % LPC, c0 = blockIdx.y * CB, col = c0 + cl;
  if (ch >= a.nseg[1]) return;
  const int4 c = a.chunk[ch];
  float2* ds = reinterpret_cast<float2*>(sm);
  float *bs = sm + 2 * SEG_CHUNK * CB, *cs = bs + SEG_CHUNK * NP;
  float a2[SPL], S[SPL];
  const size_t at = (size_t)min(col, g.C - 1) * NP + sub * SPL;
  const float* u = a.u + (size_t)ch * g.C * NP + at;
#pragma unroll
  for (int i = 0; i < SPL; ++i) { a2[i] = a.a2[at + i]; S[i] = u[i]; }
  scan_stage<T, SPL, LPC, true>(a, c, c0, act, Kp, ds, bs, cs);
  __syncthreads();
  for (int j0 = 0; j0 < c.y; j0 += TT) {
    float2 d[TT];
    float b[TT][SPL], cc[TT][SPL], y[TT];
#pragma unroll
    for (int k = 0; k < TT; ++k) { d[k] = ds[(j0 + k) * CB + cl]; lds_read<SPL>(bs + (j0 + k) * NP + sub * SPL, b[k]); lds_read<SPL>(cs + (j0 + k) * NP + sub * SPL, cc[k]); }
#pragma unroll
    for (int k = 0; k < TT; ++k) {
      y[k] = 0.0f;
#pragma unroll
      for (int i = 0; i < SPL; ++i) {
        S[i] = fmaf(hw_exp2(d[k].x * a2[i]), S[i], d[k].y * b[k][i]);
        y[k] = fmaf(S[i], cc[k][i], y[k]);
      }
    }
#pragma unroll
    for (int k = 0; k < TT; ++k) {
      const float v = lanes_sum<LPC>(y[k]);
      if (sub == 0) ds[(j0 + k) * CB + cl].x = v;              // (in the place of the step size, which only this channel's lanes read)
    }
  }
  __syncthreads();
  for (int i = tid; i < c.y * QB; i += 256) {
    const int j = i / QB, q = i % QB * 4;
    if (c0 + q >= g.Cp) continue;
    const float4* p = reinterpret_cast<const float4*>(ds + j * CB + q);
    const float y[4] = {p[0].x, p[0].z, p[1].x, p[1].z};
    scan_put4(a, c.x + j, c0 + q, y, act, Kp);
  }
}

// Decode: four states per lane, LPC = Np / 4 lanes per channel; CH (1 or 4) channels per group of lanes, CB = 256 / LPC apart, their states requested together.
// CH 4: lane i of every four takes the step size of the group's channel i.  OWN (CH 1): the third projection happens here, dtw [C][rankp] with rankp a
// multiple of 8; t in LDS.  grid (R, ceil(C / (CH CB))), block 256, LDS OWN ? rankp floats : 0.
template <typename T, int LPC, int CH, bool OWN>
__global__ __launch_bounds__(256) void k_scan_step(ScanArgs a, const T* __restrict__ dtw, int rankp, const float* __restrict__ dtb, const int32_t* __restrict__ row_active,
                                                   const int32_t* __restrict__ row_slot, const int32_t* __restrict__ row_pos, T* __restrict__ act, int Kp) {
  static_assert(CH == 1 || (CH == 4 && !OWN), "one channel per group of lanes, or one per lane of every four");
  constexpr int NP = 4 * LPC, CB = 256 / LPC;
  extern __shared__ __attribute__((aligned(16))) float ts[];
  __shared__ __attribute__((aligned(16))) float ys[CH * CB];
  const ScanGeom& g = a.g;
  const int r = blockIdx.x, tid = threadIdx.x, sub = tid % LPC, cl = tid / LPC, c0 = blockIdx.y * CB * CH;
  const int active = row_active[r], grp = row_slot[r], pos = row_pos[r];      // (requested together)
  if (!active) return;
  float4 S[CH], a2[CH];
  float* sp = a.state + ((size_t)grp * g.C) * NP + sub * 4;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int col = min(c0 + i * CB + cl, g.C - 1);
    S[i] = pos > 0 ? *reinterpret_cast<const float4*>(sp + (size_t)col * NP) : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    a2[i] = *reinterpret_cast<const float4*>(a.a2 + (size_t)col * NP + sub * 4);
  }
  float b[4] = {0.0f, 0.0f, 0.0f, 0.0f}, c[4] = {0.0f, 0.0f, 0.0f, 0.0f};
  if (sub * 4 < g.N) { a.low.at4(r, g.ob + sub * 4, b); a.low.at4(r, g.oc + sub * 4, c); }
  const int mine = min(c0 + (CH == 4 ? (tid & 3) * CB : 0) + cl, g.C - 1);
  const float x = to_f(act[act_at<T>(r, mine, Kp)]);
  float z;
  if constexpr (OWN) {
    for (int k = tid * 4; k < rankp; k += 1024) {
      float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
      if (k < g.rank) a.low.at4(r, k, v);                    // (columns behind the rank are zero up to the next multiple of 16)
      *reinterpret_cast<float4*>(ts + k) = make_float4(v[0], v[1], v[2], v[3]);
    }
    const T* wp = dtw + (size_t)mine * rankp;
    constexpr int B = 4;                                     // pieces of eight weights in flight
    float w[B][8];
#pragma unroll
    for (int i = 0; i < B; ++i)
      if ((i * LPC + sub) * 8 < rankp) load8(wp + (i * LPC + sub) * 8, w[i]);
    __syncthreads();
    z = 0.0f;
    for (int k0 = 0; k0 < rankp; k0 += B * LPC * 8) {
      if (k0 > 0) {
#pragma unroll
        for (int i = 0; i < B; ++i)
          if (k0 + (i * LPC + sub) * 8 < rankp) load8(wp + k0 + (i * LPC + sub) * 8, w[i]);
      }
#pragma unroll
      for (int i = 0; i < B; ++i) {
        const int k = k0 + (i * LPC + sub) * 8;
        if (k >= rankp) continue;
        float t[8];
        lds_read<8>(ts + k, t);
#pragma unroll
        for (int e = 0; e < 8; ++e) z = fmaf(w[i][e], t[e], z);
      }
    }
    z = lanes_sum<LPC>(z) + dtb[mine];
  } else {
    z = a.dt.at(r, mine);
  }
  const float dm = hw_softplus(z), dxm = dm * x;
#pragma unroll
  for (int i = 0; i < CH; ++i) {
    const int col = c0 + i * CB + cl;
    float d = dm, dx = dxm;
    if constexpr (CH == 4) { d = quad_lane(dm, i); dx = quad_lane(dxm, i); }
    const float4 n = make_float4(fmaf(hw_exp2(d * a2[i].x), S[i].x, dx * b[0]), fmaf(hw_exp2(d * a2[i].y), S[i].y, dx * b[1]), fmaf(hw_exp2(d * a2[i].z), S[i].z, dx * b[2]),
                                 fmaf(hw_exp2(d * a2[i].w), S[i].w, dx * b[3]));
    if (col < g.C) *reinterpret_cast<float4*>(sp + (size_t)col * NP) = n;
    const float y = lanes_sum<LPC>(fmaf(n.x, c[0], fmaf(n.y, c[1], fmaf(n.z, c[2], n.w * c[3]))));
    if (sub == 0) ys[i * CB + cl] = y;
  }
  __syncthreads();                                           // (every lane has its x)
  for (int q = tid * 4; q < CH * CB && c0 + q < g.Cp; q += 1024) scan_put4(a, r, c0 + q, ys + q, act, Kp);
}
