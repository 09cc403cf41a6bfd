// ixt_hybrid_heads.hip -- launches of attention over keys and values per head (ixt_heads_kernels.h)
#include "ixt_hybrid.h"

// k_heads_prompt / k_heads_decode: the padded (key, value) sizes they are built for, cheapest first; none fits: k_heads_any
#define IXT_HEADS_SIZES(X) X(32, 32) X(64, 64) X(64, 128) X(128, 64) X(96, 96) X(128, 128) X(192, 128) X(192, 192) X(256, 256)
// the same for two maps per head (a map has half the key size)
#define IXT_MAPS_SIZES(X) X(64, 64) X(64, 128) X(128, 64) X(128, 128) X(192, 128) X(192, 192) X(256, 128) X(256, 256)
bool heads_mfma_sizes(int d, int maps, int dv, bool f32, int* dkp, int* dvp) {
  if (f32) return false;
#define X(DK_, DV_) if (d * maps <= DK_ && dv <= DV_) { *dkp = DK_; *dvp = DV_; return true; }
  if (maps == 2) { IXT_MAPS_SIZES(X) } else { IXT_HEADS_SIZES(X) }
#undef X
  return false;
}
template <int DK, int DV, int MAPS>
static int heads_prompt_launch(HeadsAttnArgs a, hipStream_t st) {
  constexpr int lds = 2 * 64 * (DK + DV) * 2;
  static bool attr_done = false;
  if (!attr_done) {
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_heads_prompt<DK, DV, MAPS>), hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    attr_done = true;
  }
  const int GQ = a.g.H / a.g.G;
  a.HB = std::min(GQ, 64 / MAPS); a.NQ = 64 / MAPS / a.HB; a.hchunks = (GQ + a.HB - 1) / a.HB;
  hipLaunchKernelGGL((k_heads_prompt<DK, DV, MAPS>), dim3(a.g.G * a.hchunks, (a.R + a.NQ - 1) / a.NQ), dim3(256), lds, st, a);
  LAUNCHCHK();
  return IXT_OK;
}
template <int DK, int DV, int MAPS>
static int heads_launch(bool tall, bool fused, int splits, HeadsAttnArgs a, hipStream_t st) {
  if (tall) return heads_prompt_launch<DK, DV, MAPS>(a, st);
  constexpr int lds = 64 * (DK + DV) * 2;
  static bool attr_done = false;
  if (!attr_done) {
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_heads_decode<DK, DV, true, MAPS>), hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_heads_decode<DK, DV, false, MAPS>), hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    attr_done = true;
  }
  const dim3 grid(a.R, a.g.G * a.hchunks, splits);
  if (fused) hipLaunchKernelGGL((k_heads_decode<DK, DV, true, MAPS>), grid, dim3(256), lds, st, a);
  else hipLaunchKernelGGL((k_heads_decode<DK, DV, false, MAPS>), grid, dim3(256), lds, st, a);
  LAUNCHCHK();
  return IXT_OK;
}
template <typename T>
static int heads_prep(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, const HeadsRope& rope, const RowsArgs& rows, int R, hipStream_t st) {
  HybridModel* m = c->hy;
  const HeadsGeom& g = L.hg;
  const int n = g.maps * (g.H + g.G) + g.G, widest = std::max(g.dmp, g.vs);
#define HPREP(LP_) hipLaunchKernelGGL((k_heads_prep<T, LP_>), dim3(R, (n * LP_ + 255) / 256), dim3(256), 0, st, t, g, W.qn, W.kn, m->eps, rope, rows, (T*)L.pages, (T*)L.vpages, (T*)m->qx)
  if (widest <= 64) HPREP(16); else if (widest <= 128) HPREP(32); else HPREP(64);
#undef HPREP
  LAUNCHCHK();
  return IXT_OK;
}
// how the keys of a launch over few rows are split: at least a tile each
static int heads_splits(const HeadsGeom& g, int R, int hchunks, int len_hint) {
  const int blocks = R * g.G * hchunks, most = g.chunk > 0 ? g.chunk : g.window, span = most > 0 ? std::min(most, len_hint) : len_hint;
  return std::min(std::min(16, std::max(1, IXT_HEADS_SPLIT_BLOCKS / blocks)), std::max(1, (span + 63) / 64));
}
static HeadsAttnArgs heads_args(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, int R) {
  HybridModel* m = c->hy;
  const HeadsGeom& g = L.hg;
  const int GQ = g.H / g.G, hchunks = (GQ * g.maps + 15) / 16;
  return HeadsAttnArgs{(const bf16_t*)m->qx, g, W.sink, RowsArgs{c->row_slot, c->row_pos, c->row_active, c->ps.page_map}, (bf16_t*)L.pages, (bf16_t*)L.vpages, R, 1, (GQ + hchunks - 1) / hchunks, hchunks,
                       __builtin_ctz(c->P), (bf16_t*)m->act, W.okp, m->po, m->pml, t, W.qn, W.kn, m->eps, HeadsRope{L.rope_cos, L.rope_sin}, MapsArgs{W.lambda, 1.0f - L.c.map_diff, m->eps}};
}
template <int DK, int DV>
static int pair_launch(const HeadsAttnArgs& a, int splits, const RetArgs& b, const HeadsRope& rope, hipStream_t st) {
  constexpr int lds = 64 * (DK + DV) * 2;
  const size_t need = std::max((size_t)lds, ret_step_lds(b.g));
  static size_t most = 0;
  if (need > most) {
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_pair_decode<DK, DV>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)need));
    most = need;
  }
  hipLaunchKernelGGL((k_pair_decode<DK, DV>), dim3(a.R * (b.g.H + a.g.G * a.hchunks * splits)), dim3(256), need, st, a, splits, b, rope, a.Kp);
  LAUNCHCHK();
  return IXT_OK;
}
template <>
int heads_beside_retention<float>(ixt_ctx*, const HLayer&, const HLayer&, const Slices&, int, int, hipStream_t, bool* done) { *done = false; return IXT_OK; }
template <>
int heads_beside_retention<bf16_t>(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, int R, int len_hint, hipStream_t st, bool* done) {
  const HeadsGeom& g = L.hg;
  int dkp = 0, dvp = 0;
  *done = L.c.mixer == IXT_MIX_ATTENTION && L.side && L.side->c.mixer != IXT_MIX_ATTENTION && R <= 32 && g.maps == 1 && heads_mfma_sizes(g.d, 1, g.dv, false, &dkp, &dvp);
  if (!*done) return IXT_OK;
  const HeadsAttnArgs a = heads_args(c, L, W, t, R);
  const RetArgs b = ret_args(c->hy, *L.side, t.from(L.side->c0));
  const HeadsRope rope{L.side->rope_cos, L.side->rope_sin};
  const int splits = heads_splits(g, R, a.hchunks, len_hint);
  int rc = IXT_ERR_UNSUPPORTED;
#define X(DK_, DV_) if (dkp == DK_ && dvp == DV_) rc = pair_launch<DK_, DV_>(a, splits, b, rope, st);
  IXT_HEADS_SIZES(X)
#undef X
  TRY(rc);
  const float* w = W.side->onorm;
  if (splits > 1 && b.g.join_norm) hipLaunchKernelGGL(k_pair_join, dim3(R, g.H + 1), dim3(256), 0, st, a, splits, b, w, a.Kp);
  else if (splits > 1) hipLaunchKernelGGL(k_heads_combine, dim3(R, g.H), dim3(64), 0, st, a.part_o, a.part_ml, splits, g, a.mp, t, c->row_active, a.out, a.Kp);
  else if (b.g.join_norm) hipLaunchKernelGGL((k_ret_join<bf16_t>), dim3(R), dim3(256), 0, st, b, w, c->row_active, a.out, a.Kp);
  LAUNCHCHK();
  return IXT_OK;
}
// attention of a layer over heads: projection t -> pages, and the operand of the output projection in m->act.  L: the layer, W: the one with its parameters
template <typename T>
int heads_attention(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, int R, bool decode, int len_hint, hipStream_t st) {
  HybridModel* m = c->hy;
  const HeadsGeom& g = L.hg;
  const RowsArgs rows{c->row_slot, c->row_pos, c->row_active, c->ps.page_map};
  const HeadsRope rope{L.rope_cos, L.rope_sin};
  const MapsArgs mp{W.lambda, 1.0f - L.c.map_diff, m->eps};
  int dkp = 0, dvp = 0;
  if constexpr (sizeof(T) == 2) {
    if (heads_mfma_sizes(g.d, g.maps, g.dv, m->f32, &dkp, &dvp)) {
      const bool tall = !decode && R > 32;
      if (!decode) TRY((heads_prep<T>(c, L, W, t, rope, rows, R, st)));
      const HeadsAttnArgs a = heads_args(c, L, W, t, R);
      const int splits = tall ? 1 : heads_splits(g, R, a.hchunks, len_hint);
      int rc = IXT_ERR_UNSUPPORTED;
#define X(DK_, DV_) if (dkp == DK_ && dvp == DV_) rc = heads_launch<DK_, DV_, 1>(tall, decode, splits, a, st);
#define X2(DK_, DV_) if (dkp == DK_ && dvp == DV_) rc = heads_launch<DK_, DV_, 2>(tall, decode, splits, a, st);
      if (g.maps == 2) { IXT_MAPS_SIZES(X2) } else { IXT_HEADS_SIZES(X) }
#undef X2
#undef X
      TRY(rc);
      if (splits > 1) {
        hipLaunchKernelGGL(k_heads_combine, dim3(R, g.H), dim3(64), 0, st, m->po, m->pml, splits, g, mp, t, c->row_active, (bf16_t*)m->act, W.okp);
        LAUNCHCHK();
      }
      return IXT_OK;
    }
  }
  TRY((heads_prep<T>(c, L, W, t, rope, rows, R, st)));
  hipLaunchKernelGGL((k_heads_any<T>), dim3(R, g.H), dim3(256), sizeof(float) * (g.dkp + 256), st, (const T*)m->qx, g, W.sink, rows, (const T*)L.pages, (const T*)L.vpages, mp, t, (T*)m->act,
                     W.okp);
  LAUNCHCHK();
  return IXT_OK;
}
template int heads_attention<bf16_t>(ixt_ctx*, const HLayer&, const HLayer&, const Slices&, int, bool, int, hipStream_t);
template int heads_attention<float>(ixt_ctx*, const HLayer&, const HLayer&, const Slices&, int, bool, int, hipStream_t);
