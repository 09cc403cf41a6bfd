// ixt_scan_kernels.h -- selective scan (IXT_MIX_SCAN): per channel c and state n
//   S <- exp(dt_c A[c, n]) S + dt_c x_c B_n,   y_c = sum_n S[c, n] C_n + D_c x_c,   output y silu(z),
// dt = softplus(projection + bias), A = -exp(A_log); x behind a short causal convolution with bias and silu.  Everything from dt on is f32; the state
// [group][C][Np] lives as long as its page group.
//
// Over a run of rows the recurrence goes by chunks of SEG_CHUNK rows (k_segments lists them): the state behind a chunk is exp(A sum dt) times the one in
// front of it plus what the chunk leaves by itself.
//
//   k_scan_conv   projection slices -> x in f32 and as the operand of the next projection
//   k_scan_rank   the step-size part of that projection as the operand of the third one
//   k_scan_sums   chunk by chunk: U = the state a chunk leaves from zero, and its sum of dt
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
  const float *a2, *D;                      // [C][Np]: -exp(A_log) log2(e), zeros behind N; [Cp]
  const int32_t* seg; const int4* chunk; const int32_t* nseg;
  const float* x;                           // [R][Cp]
  float *u, *sum, *state;                   // [chunk][C][Np], [chunk][Cp], [group][C][Np]
};

// a2 in place from A_log.  Padding stays zero.
static __global__ __launch_bounds__(256) void k_scan_rates(float* __restrict__ a2, int C, int N, int Np) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < C * Np && i % Np < N) a2[i] = -1.44269504088896340736f * expf(a2[i]);
}

// grid (R, ceil(Kp / 256)), block 256: a channel per thread.  tails [group][2][taps - 1][C].
struct ScanConvArgs {
  Slices t; ScanGeom g; const float *w, *bias; const int32_t *row_seg, *row_j, *seg;
  float *tails, *x;
};
template <typename T>
__global__ __launch_bounds__(256) void k_scan_conv(ScanConvArgs a, T* __restrict__ out, int Kp) {
  const ScanGeom& g = a.g;
  const int r = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x, s = a.row_seg[r];
  if (s < 0 || c >= Kp) return;
  float v = 0.0f;
  if (c < g.C) {
    const int32_t* sg = a.seg + (size_t)s * 8;
    const size_t tsz = (size_t)(g.taps - 1) * g.C;
    float* tb = a.tails + (size_t)sg[2] * 2 * tsz;
    const ConvCtx cc{tb + (size_t)sg[4] * tsz, tb + (size_t)(sg[4] ^ 1) * tsz, a.row_j[r], sg[1], sg[3]};
    v = conv_channel(a.t, r, c, a.w + (size_t)c * g.taps, g.taps, c, g.C, cc) + a.bias[c];
    v *= f32_sigmoid(v);
  }
  if (c < g.Cp) a.x[(size_t)r * g.Cp + c] = v;
  act_store1(out, r, c, Kp, v);
}

// grid (R), block 128
template <typename T>
__global__ __launch_bounds__(128) void k_scan_rank(Slices low, int rank, T* __restrict__ out, int Kp) {
  for (int k = threadIdx.x; k < Kp; k += 128) act_store1(out, blockIdx.x, k, Kp, k < rank ? low.at(blockIdx.x, k) : 0.0f);
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

// A chunk's operands -> LDS: step sizes and inputs [SEG_CHUNK][CB] of CB channels from c0 on, the B (and C) columns [SEG_CHUNK][Np]
template <int SPL, int LPC, bool OUT>
__device__ __forceinline__ void scan_stage(const ScanArgs& a, const int4& c, int c0, float* dts, float* xs, float* bs, float* cs) {
  constexpr int CB = 256 / LPC, NP = SPL * LPC, QB = CB / 4, QN = NP / 4;
  const ScanGeom& g = a.g;
  const int tid = threadIdx.x, n = c.y;
  for (int i = tid; i < SEG_CHUNK * QB; i += 256) {
    const int j = i / QB, q = i % QB * 4, ch = c0 + q;
    float d[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    float4 x = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (j < n && ch < g.Cp) {                                // (columns C .. Cp - 1 of both are zero projections; a2 and D are zero there)
      a.dt.at4(c.x + j, ch, d);
      x = *reinterpret_cast<const float4*>(a.x + (size_t)(c.x + j) * g.Cp + ch);
#pragma unroll
      for (int e = 0; e < 4; ++e) d[e] = f32_softplus(d[e]);
    }
    *reinterpret_cast<float4*>(dts + j * CB + q) = make_float4(d[0], d[1], d[2], d[3]);
    *reinterpret_cast<float4*>(xs + j * CB + q) = x;
  }
  for (int i = tid; i < SEG_CHUNK * QN; i += 256) {
    const int j = i / QN, q = i % QN * 4;
    float b[4] = {0.0f, 0.0f, 0.0f, 0.0f}, y[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (j < n)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (q + e < g.N) {
          b[e] = a.low.at(c.x + j, g.ob + q + e);
          if (OUT) y[e] = a.low.at(c.x + j, g.oc + q + e);
        }
    *reinterpret_cast<float4*>(bs + j * NP + q) = make_float4(b[0], b[1], b[2], b[3]);
    if (OUT) *reinterpret_cast<float4*>(cs + j * NP + q) = make_float4(y[0], y[1], y[2], y[3]);
  }
}
template <int SPL, int LPC, bool OUT> constexpr size_t scan_lds() { return sizeof(float) * SEG_CHUNK * (2 * (256 / LPC) + (OUT ? 2 : 1) * SPL * LPC); }

// grid (chunks, ceil(C / CB)), block 256, LDS scan_lds<SPL, LPC, false>()
template <int SPL, int LPC>
__global__ __launch_bounds__(256) void k_scan_sums(ScanArgs a) {
  constexpr int CB = 256 / LPC, NP = SPL * LPC;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const ScanGeom& g = a.g;
  const int ch = blockIdx.x, tid = threadIdx.x, cl = tid / LPC, sub = tid % LPC, c0 = blockIdx.y * CB, col = c0 + cl;
  if (ch >= a.nseg[1]) return;
  const int4 c = a.chunk[ch];
  float *dts = sm, *xs = dts + SEG_CHUNK * CB, *bs = xs + SEG_CHUNK * CB;
  float a2[SPL], S[SPL];
  const size_t at = (size_t)min(col, g.C - 1) * NP + sub * SPL;
#pragma unroll
  for (int i = 0; i < SPL; ++i) { a2[i] = a.a2[at + i]; S[i] = 0.0f; }
  scan_stage<SPL, LPC, false>(a, c, c0, dts, xs, bs, nullptr);
  __syncthreads();
  float sum = 0.0f;
  for (int j = 0; j < c.y; ++j) {
    const float dt = dts[j * CB + cl], dx = dt * xs[j * CB + cl];
    const float* b = bs + j * NP + sub * SPL;
    sum += dt;
#pragma unroll
    for (int i = 0; i < SPL; ++i) S[i] = fmaf(hw_exp2(dt * a2[i]), S[i], dx * b[i]);
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

// outputs -> act.  grid (chunks, ceil(max(C, Kp) / CB)), block 256, LDS scan_lds<SPL, LPC, true>()
template <typename T, int SPL, int LPC>
__global__ __launch_bounds__(256) void k_scan_out(ScanArgs a, T* __restrict__ out, int Kp) {
  constexpr int CB = 256 / LPC, NP = SPL * LPC, QB = CB / 4;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const ScanGeom& g = a.g;
  const int ch = blockIdx.x, tid = threadIdx.x, cl = tid / LPC, sub = tid % LPC, c0 = blockIdx.y * CB, col = c0 + cl;
  if (ch >= a.nseg[1]) return;
  const int4 c = a.chunk[ch];
  float *dts = sm, *xs = dts + SEG_CHUNK * CB, *bs = xs + SEG_CHUNK * CB, *cs = bs + SEG_CHUNK * NP;
  if (c0 < g.C) {
    float a2[SPL], S[SPL];
    const size_t at = (size_t)min(col, g.C - 1) * NP + sub * SPL;
    const float* u = a.u + (size_t)ch * g.C * NP + at;
#pragma unroll
    for (int i = 0; i < SPL; ++i) { a2[i] = a.a2[at + i]; S[i] = u[i]; }
    const float D = a.D[min(col, g.C - 1)];
    scan_stage<SPL, LPC, true>(a, c, c0, dts, xs, bs, cs);
    __syncthreads();
    for (int j = 0; j < c.y; ++j) {
      const float dt = dts[j * CB + cl], x = xs[j * CB + cl], dx = dt * x;
      const float *b = bs + j * NP + sub * SPL, *cc = cs + j * NP + sub * SPL;
      float y = 0.0f;
#pragma unroll
      for (int i = 0; i < SPL; ++i) {
        S[i] = fmaf(hw_exp2(dt * a2[i]), S[i], dx * b[i]);
        y = fmaf(S[i], cc[i], y);
      }
      y = lanes_sum<LPC>(y);
      if (sub == 0) dts[j * CB + cl] = fmaf(D, x, y);          // (in the place of its step size, which only this channel's lanes read)
    }
    __syncthreads();
  }
  for (int i = tid; i < c.y * QB; i += 256) {
    const int j = i / QB, q = i % QB * 4, col4 = c0 + q;
    if (col4 >= Kp) continue;
    float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    if (col4 < g.C) {
      const float4 y = *reinterpret_cast<const float4*>(dts + j * CB + q);
      float z[4];
      a.in.at4(c.x + j, g.oz + col4, z);
      v[0] = y.x * z[0] * f32_sigmoid(z[0]); v[1] = y.y * z[1] * f32_sigmoid(z[1]); v[2] = y.z * z[2] * f32_sigmoid(z[2]); v[3] = y.w * z[3] * f32_sigmoid(z[3]);
    }
    act_store4(out, c.x + j, col4, Kp, v);
  }
}

// Decode: four states per lane, LPC = Np / 4 lanes per channel.  grid (R, ceil(max(C, Kp) / (256 / LPC))), block 256.
template <typename T, int LPC>
__global__ __launch_bounds__(256) void k_scan_step(ScanArgs a, const int32_t* __restrict__ row_active, const int32_t* __restrict__ row_slot, const int32_t* __restrict__ row_pos,
                                                   T* __restrict__ out, int Kp) {
  constexpr int NP = 4 * LPC;
  const ScanGeom& g = a.g;
  const int r = blockIdx.x, tid = threadIdx.x, sub = tid % LPC, col = blockIdx.y * (256 / LPC) + tid / LPC;
  const int active = row_active[r], grp = row_slot[r], pos = row_pos[r];      // (requested together)
  if (!active) return;
  if (col >= g.C) {
    if (col < Kp && sub == 0) act_store1(out, r, col, Kp, 0.0f);
    return;
  }
  float4* sp = reinterpret_cast<float4*>(a.state + ((size_t)grp * g.C + col) * NP + sub * 4);
  const float4 S0 = pos > 0 ? *sp : make_float4(0.0f, 0.0f, 0.0f, 0.0f), a2 = *reinterpret_cast<const float4*>(a.a2 + (size_t)col * NP + sub * 4);
  const float x = a.x[(size_t)r * g.Cp + col], z = a.in.at(r, g.oz + col), D = a.D[col], dt = f32_softplus(a.dt.at(r, col)), dx = dt * x;
  float b[4] = {0.0f, 0.0f, 0.0f, 0.0f}, c[4] = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (sub * 4 + e < g.N) { b[e] = a.low.at(r, g.ob + sub * 4 + e); c[e] = a.low.at(r, g.oc + sub * 4 + e); }
  const float4 S = make_float4(fmaf(hw_exp2(dt * a2.x), S0.x, dx * b[0]), fmaf(hw_exp2(dt * a2.y), S0.y, dx * b[1]), fmaf(hw_exp2(dt * a2.z), S0.z, dx * b[2]),
                               fmaf(hw_exp2(dt * a2.w), S0.w, dx * b[3]));
  *sp = S;
  const float y = lanes_sum<LPC>(fmaf(S.x, c[0], fmaf(S.y, c[1], fmaf(S.z, c[2], S.w * c[3]))));
  if (sub == 0) act_store1(out, r, col, Kp, fmaf(D, x, y) * z * f32_sigmoid(z));
}
