// ixt_hybrid_norm.hip -- launches of the norms between sublayers and in front of the head (every padded width, norm kind and number of streams)
#include "ixt_hybrid.h"

// x <- x + post(t), the next operand pre(x), or the same among streams (k_sub_norm); routed: its f32 copy too.  A token shift behind pre is part of the launch
// where a row needs no other row of it (single), a launch of its own otherwise
template <typename T>
int hybrid_norm(ixt_ctx* c, const SubOut& o, const Around& ar, bool routed, int R, bool single, hipStream_t st) {
  HybridModel* m = c->hy;
  const bool later = ar.mu != nullptr && !single;
  float* h32 = (routed || later) && ar.pre.w != nullptr ? m->h32 : nullptr;
  T* to = later ? nullptr : (T*)(ar.to_cat ? m->cat : m->xb);
  const ShiftArgs sh = ar.mu != nullptr && single ? ShiftArgs{ar.mu, ar.shift, c->row_slot, c->row_pos, c->row_active, m->parity} : ShiftArgs{};
  const HyperW hc{ar.hc_next, ar.hc ? ar.hc + HC_MAX : nullptr, ar.hc ? ar.hc + 2 * HC_MAX : nullptr};
  const SubNormArgs a{o.t, o.add, o.addw, o.pos, o.wts, o.top, ar.post, ar.pre, m->eps, m->E, m->Ep, m->streams, hc, o.bias, o.fbias, o.fresh ? 1 : 0, sh, ar.to_cat ? 2 * m->Ep : m->Ep};
#define HNORM_S(NI_, KIND_, SM_) hipLaunchKernelGGL((k_sub_norm<T, NI_, KIND_, SM_>), dim3(R), dim3(256), 0, st, a, m->x, to, h32)
#define HNORM(NI_, KIND_) do { if (m->streams == 0) HNORM_S(NI_, KIND_, 0); else if (m->streams <= 4) HNORM_S(NI_, KIND_, 4); else HNORM_S(6, KIND_, HC_MAX); } while (0)
#define HNORM_K(NI_) do { if (m->norm_kind == IXT_NORM_TANH) HNORM(NI_, IXT_NORM_TANH); else if (m->norm_kind == IXT_NORM_LAYER) HNORM(NI_, IXT_NORM_LAYER); else if (m->norm_kind == IXT_NORM_ONE) HNORM(NI_, IXT_NORM_ONE); else HNORM(NI_, IXT_NORM_RMS); } while (0)
  if (m->Ep <= 2048) HNORM_K(1); else if (m->Ep <= 4096) HNORM_K(2); else if (m->Ep <= 8192) HNORM_K(4); else HNORM_K(6);
#undef HNORM_K
#undef HNORM
#undef HNORM_S
  LAUNCHCHK();
  if (later) {
    hipLaunchKernelGGL((k_token_shift<T>), dim3(R), dim3(256), 0, st, m->h32, ar.mu, ar.shift, m->row_seg, m->row_j, m->seg, m->E, m->Ep, (T*)m->xb);
    LAUNCHCHK();
  }
  return IXT_OK;
}

// rows lrows[i] (or lrow0 + i), n of them, of the residual stream -> the model's norm -> the head's operand
template <typename T>
int hybrid_final_norm(ixt_ctx* c, int R, int n, const int32_t* lrows, int lrow0, hipStream_t st) {
  HybridModel* m = c->hy;
#define HFINAL(NI_, KIND_) hipLaunchKernelGGL((k_final_norm<T, NI_, KIND_>), dim3(n), dim3(256), 0, st, m->x, lrows, lrow0, R, std::max(1, m->streams), \
                                              m->fnorm, m->eps, m->E, m->Ep, (T*)m->xn)
#define HFINAL_K(NI_) do { if (m->norm_kind == IXT_NORM_TANH) HFINAL(NI_, IXT_NORM_TANH); else if (m->norm_kind == IXT_NORM_LAYER) HFINAL(NI_, IXT_NORM_LAYER); else if (m->norm_kind == IXT_NORM_ONE) HFINAL(NI_, IXT_NORM_ONE); else HFINAL(NI_, IXT_NORM_RMS); } while (0)
  if (m->Ep <= 2048) HFINAL_K(1); else if (m->Ep <= 4096) HFINAL_K(2); else if (m->Ep <= 8192) HFINAL_K(4); else HFINAL_K(6);
#undef HFINAL_K
#undef HFINAL
  LAUNCHCHK();
  return IXT_OK;
}
template int hybrid_norm<bf16_t>(ixt_ctx*, const SubOut&, const Around&, bool, int, bool, hipStream_t);
template int hybrid_norm<float>(ixt_ctx*, const SubOut&, const Around&, bool, int, bool, hipStream_t);
template int hybrid_final_norm<bf16_t>(ixt_ctx*, int, int, const int32_t*, int, hipStream_t);
template int hybrid_final_norm<float>(ixt_ctx*, int, int, const int32_t*, int, hipStream_t);
