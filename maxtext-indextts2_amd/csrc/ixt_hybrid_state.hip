// ixt_hybrid_state.hip -- launches of the mixers whose state is a recurrence over chunks of rows: retention (ixt_retention_kernels.h), selective scan
// (ixt_scan_kernels.h)
#include "ixt_hybrid.h"

template <int NT, bool FUSED, typename T>
static int ret_out_launch(const RetArgs& a, int chunks, T* out, int Kp, hipStream_t st) {
  hipLaunchKernelGGL((k_ret_out<T, NT, FUSED>), dim3(chunks, a.g.H, (a.g.dvp + 16 * NT - 1) / (16 * NT)), dim3(256), 0, st, a, out, Kp);
  LAUNCHCHK();
  return IXT_OK;
}
template <typename T>
int retention_mix(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, int R, int nseg_max, bool single, hipStream_t st) {
  HybridModel* m = c->hy;
  const RetGeom& g = L.rg;
  const RowsArgs rows{c->row_slot, c->row_pos, c->row_active, c->ps.page_map};
  const HeadsRope rope{L.rope_cos, L.rope_sin};
  const RetArgs a = ret_args(m, L, t);
  T* out = (T*)m->act;
  const int Kp = W.okp;
  if (single) {            // every row is a run of one token
    hipLaunchKernelGGL((k_ret_step<T>), dim3(R, g.H), dim3(256), ret_step_lds(g), st, a, rope, rows, out, Kp);
  } else {
    const int widest = std::max(g.dp, g.dvp), chunks = R / SEG_CHUNK + nseg_max;
#define RPREP(LP_) hipLaunchKernelGGL((k_ret_prep<LP_>), dim3(R, (3 * g.H * LP_ + 255) / 256), dim3(256), 0, st, a, rope, rows)
    if (widest <= 64) RPREP(16); else if (widest <= 128) RPREP(32); else RPREP(64);
#undef RPREP
    hipLaunchKernelGGL(k_ret_sums, dim3(chunks, g.H, (g.dp + 63) / 64 * ((g.dvp + 127) / 128)), dim3(256), 0, st, a);
    hipLaunchKernelGGL(k_ret_carry, dim3(nseg_max, g.H, (g.dp * g.dvp + 1023) / 1024), dim3(256), 0, st, a);
    LAUNCHCHK();
    if (g.join_norm) TRY(g.dvp <= 32 ? (ret_out_launch<2, false, T>(a, chunks, out, Kp, st)) : g.dvp <= 64 ? (ret_out_launch<4, false, T>(a, chunks, out, Kp, st)) : (ret_out_launch<8, false, T>(a, chunks, out, Kp, st)));
    else if (g.dvp <= 32) return ret_out_launch<2, true, T>(a, chunks, out, Kp, st);
    else if (g.dvp <= 64) return ret_out_launch<4, true, T>(a, chunks, out, Kp, st);
    else if (g.dvp <= 128) return ret_out_launch<8, true, T>(a, chunks, out, Kp, st);
    else {
      TRY((ret_out_launch<8, false, T>(a, chunks, out, Kp, st)));
      hipLaunchKernelGGL((k_ret_gate<T>), dim3(R, (g.H + 3) / 4), dim3(256), 0, st, a, c->row_active, out, Kp);
    }
  }
  if (g.join_norm) hipLaunchKernelGGL((k_ret_join<T>), dim3(R), dim3(256), 0, st, a, W.onorm, c->row_active, out, Kp);
  LAUNCHCHK();
  return IXT_OK;
}
template int retention_mix<bf16_t>(ixt_ctx*, const HLayer&, const HLayer&, const Slices&, int, int, bool, hipStream_t);
template int retention_mix<float>(ixt_ctx*, const HLayer&, const HLayer&, const Slices&, int, int, bool, hipStream_t);

template <typename T>
int scan_conv(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& in, int R, hipStream_t st) {
  HybridModel* m = c->hy;
  const ScanConvArgs a{in, L.sg, W.cw, W.cb, m->row_seg, m->row_j, m->seg, L.tails, R};
  const unsigned cols = (W.okp + 1023) / 1024;
  if (R >= 256) hipLaunchKernelGGL((k_scan_conv<T, 4>), dim3((R + 3) / 4, cols), dim3(256), 0, st, a, (T*)m->act, W.okp);
  else hipLaunchKernelGGL((k_scan_conv<T, 1>), dim3(R, cols), dim3(256), 0, st, a, (T*)m->act, W.okp);
  LAUNCHCHK();
  return IXT_OK;
}
template <typename T>
int scan_rank(ixt_ctx* c, const HLayer& W, const Slices& low, int R, hipStream_t st) {
  hipLaunchKernelGGL((k_scan_rank<T>), dim3(R), dim3(64), 0, st, low, c->hy->part2, W.sg.rank, (T*)c->hy->scan_t, W.dt.Kp);
  LAUNCHCHK();
  return IXT_OK;
}
template <typename T, int SPL, int LPC>
static int scan_chunks(ixt_ctx* c, const ScanArgs& a, int R, int nseg_max, int Kp, hipStream_t st) {
  static bool attr_done = false;
  if (!attr_done) {
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_scan_sums<T, SPL, LPC>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)scan_lds<SPL, LPC, false>()));
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_scan_out<T, SPL, LPC>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)scan_lds<SPL, LPC, true>()));
    attr_done = true;
  }
  constexpr int CB = 256 / LPC;
  const ScanGeom& g = a.g;
  const int chunks = R / SEG_CHUNK + nseg_max;
  hipLaunchKernelGGL((k_scan_sums<T, SPL, LPC>), dim3(chunks, (g.C + CB - 1) / CB), dim3(256), (scan_lds<SPL, LPC, false>()), st, a, (const T*)c->hy->act, Kp);
  hipLaunchKernelGGL(k_scan_carry, dim3(nseg_max, (unsigned)(((size_t)g.C * g.Np + 1023) / 1024)), dim3(256), 0, st, a);
  hipLaunchKernelGGL((k_scan_out<T, SPL, LPC>), dim3(chunks, (g.C + CB - 1) / CB), dim3(256), (scan_lds<SPL, LPC, true>()), st, a, (T*)c->hy->act, Kp);
  LAUNCHCHK();
  return IXT_OK;
}
template <typename T>
int scan_mix(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& in, const Slices& low, const Slices& dt, int R, int nseg_max, bool single, hipStream_t st) {
  HybridModel* m = c->hy;
  const ScanGeom& g = L.sg;
  const ScanArgs a{g, in, low, dt, m->part3, W.a2, W.D, m->seg, m->chunk, m->nseg, m->scan_u, m->scan_sum, L.state};
  const int Kp = W.okp;
  if (single) {
#define SSTEP_C(LPC_, CH_, OWN_) hipLaunchKernelGGL((k_scan_step<T, LPC_, CH_, OWN_>), dim3(R, (g.C * LPC_ + 256 * CH_ - 1) / (256 * CH_)), dim3(256), OWN_ ? sizeof(float) * W.rankp : 0, st, a, \
                                                    (const T*)W.dtw, W.rankp, W.dtb, c->row_active, c->row_slot, c->row_pos, (T*)m->act, Kp)
#define SSTEP(LPC_) case 4 * LPC_: if (dt.p == nullptr) SSTEP_C(LPC_, 1, true); else if (R * (size_t)g.C * LPC_ >= 256 * 4096) SSTEP_C(LPC_, 4, false); else SSTEP_C(LPC_, 1, false); break
    switch (g.Np) { SSTEP(4); SSTEP(8); SSTEP(16); SSTEP(32); SSTEP(64); default: return set_err(IXT_ERR_UNSUPPORTED, "selective scan: %d states", g.N); }
#undef SSTEP
#undef SSTEP_C
    LAUNCHCHK();
    return IXT_OK;
  }
  switch (g.Np) {
    case 16: return scan_chunks<T, 4, 4>(c, a, R, nseg_max, Kp, st);      // (8 states on two lanes: 44 against 28 us)
    case 32: return scan_chunks<T, 8, 4>(c, a, R, nseg_max, Kp, st);
    case 64: return scan_chunks<T, 16, 4>(c, a, R, nseg_max, Kp, st);
    case 128: return scan_chunks<T, 16, 8>(c, a, R, nseg_max, Kp, st);
    case 256: return scan_chunks<T, 16, 16>(c, a, R, nseg_max, Kp, st);
    default: return set_err(IXT_ERR_UNSUPPORTED, "selective scan: %d states", g.N);
  }
}
#define SCAN_T(T) \
  template int scan_conv<T>(ixt_ctx*, const HLayer&, const HLayer&, const Slices&, int, hipStream_t); \
  template int scan_rank<T>(ixt_ctx*, const HLayer&, const Slices&, int, hipStream_t); \
  template int scan_mix<T>(ixt_ctx*, const HLayer&, const HLayer&, const Slices&, const Slices&, const Slices&, int, int, bool, hipStream_t);
SCAN_T(bf16_t)
SCAN_T(float)
