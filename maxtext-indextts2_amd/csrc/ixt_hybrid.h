// ixt_hybrid.h -- what the host objects of hybrid decoders share: the model, its layer plans, and the launch helpers that live in objects of their own
// (they compile side by side): norms between sublayers (ixt_hybrid_norm.hip), attention over heads (ixt_hybrid_heads.hip), retention and selective scan
// (ixt_hybrid_state.hip).
#pragma once
#include "ixt_internal.h"
#include "ixt_heads_kernels.h"
#include "ixt_hybrid_kernels.h"
#include "ixt_retention_kernels.h"
#include "ixt_scan_kernels.h"

#include <memory>

struct HMat { void* w = nullptr; int K = 0, N = 0, Kp = 0, Np = 0; };       // a dot operand of the ctx's storage type, zero-padded
struct HLayer {
  ixt_layer c{};
  int src = 0;                                   // the layer whose parameters are used
  LatentGeom lg{};
  DeltaGeom dg{};
  HeadsGeom hg{};
  RetGeom rg{};
  ScanGeom sg{};
  HMat in, low, o, gu, down;                     // input projection, second low-rank product (scan: x -> [t | B | C]), output projection, gate | up (or up), down
  HMat dt;                                       // scan: t -> step sizes, and the same row by row [channel][rankp] for few rows
  void* dtw = nullptr;
  int rankp = 0;
  std::unique_ptr<HLayer> side;                  // the mixer beside this one: its geometry, parameters, caches and state; columns of the same `in` and `o`
  int in_cols = 0, o_rows = 0;                   // columns of `in`, rows of `o` (a side mixer: its own)
  int c0 = 0, okp = 0;                           // first column of `in` that is this mixer's; columns of a row of the output projection's operand
  float *ibias = nullptr, *obias = nullptr;      // biases per column of `in` (kept by the mixer that owns it), of the output projection
  float *mu = nullptr, *shift = nullptr;         // token shift: its numbers, the groups' last h (ShiftArgs)
  HMat uq;                                       // latent layer: the queries' up-projection (none: they are columns of `in`)
  HMat uk, uv;                                   // per-head matrices of a latent layer (heads * wstride elements apart): d -> rank, rank -> v
  int d_off = 0, g_off = 0;                      // latent layer: columns of the latent and of the output gate in the input projection
  size_t uk_stride = 0, uv_stride = 0, gu_stride = 0, down_stride = 0;
  NormW n1{}, n1b{}, n2{}, n2b{};                // in front of / behind the mixer, in front of / behind the feed-forward
  HMat sgu, sdown;                               // a mixture's shared unit
  float *hc1 = nullptr, *hc2 = nullptr;          // hyper-connections: [HC_MAX] in, [HC_MAX] out, [HC_MAX][HC_MAX] mix
  float *qnorm = nullptr, *maps = nullptr, *lambda = nullptr, *bias = nullptr, *pow = nullptr;      // query latent's norm; lq1, lk1, lq2, lk2 and their number; router bias; powers of the decays
  float *qn = nullptr, *kn = nullptr, *sink = nullptr, *corr = nullptr;
  float *cnorm = nullptr, *cq = nullptr, *ck = nullptr, *cv = nullptr, *a_log = nullptr, *dt_bias = nullptr, *onorm = nullptr, *router = nullptr;
  float *a2 = nullptr, *D = nullptr, *dtb = nullptr, *cw = nullptr, *cb = nullptr;      // scan: rates, skip, step-size bias, convolution and its bias
  float *unit = nullptr, *unit_par = nullptr;    // xIELU: the tensor, its numbers
  const float *rope_cos = nullptr, *rope_sin = nullptr;
  void* pages = nullptr;                         // latent layer: [page][token][rankp + rotp]; attention layer: keys [page][kv head][token][dkp]
  void* vpages = nullptr;                        // attention layer: values [page][kv head][token][dvp]
  float *state = nullptr, *tails = nullptr;      // delta layer: [group][H][dv][dp], [group][2][taps - 1][C]; retention: [group][H][dp][dvp]; scan: [group][C][Np], [group][2][taps - 1][C]
};
struct HTensor { std::vector<int64_t> shape; std::function<int(const void*, int, hipStream_t)> load; bool done = false; };   // load empty: accepted, unused
struct HybridModel {
  bool f32 = false, recurrent = false;
  size_t esz = 2;                                // bytes per activation / weight element
  int E = 0, Ep = 0, V = 0, maxH = 0, kmax_pad = 0, norm_kind = 0, norm_places = 0, streams = 0;      // maxH: most heads of a latent layer
  bool tied = false;                             // the head is the embedding table
  float emb_scale = 1.0f, logit_scale = 1.0f, eps = 1e-5f;
  std::vector<HLayer> layers;
  std::map<std::string, HTensor> tensors;
  size_t missing = 0;
  void* embed = nullptr;
  HMat head;
  NormW fnorm{};
  int passes = 0;                                // passes of the loop (0: there is none)
  HMat loop_in;
  float* loop_step = nullptr;                    // [passes][Ep]
  // workspaces
  float *x = nullptr, *part2 = nullptr, *h32 = nullptr;      // h32: a routed layer's normed input in f32
  size_t part2_floats = 0;
  void *cat = nullptr;                           // a loop: act of [x | embedding output], Ep columns each
  void* scan_t = nullptr;                        // the operand of a scan's third projection
  float *part3 = nullptr, *scan_u = nullptr, *scan_sum = nullptr;
  size_t part3_floats = 0;
  void *xb = nullptr, *act = nullptr, *hact = nullptr, *xn = nullptr, *qx = nullptr, *qr = nullptr, *olat = nullptr, *xg = nullptr, *mhact = nullptr;
  float *dq = nullptr, *dk = nullptr, *dkq = nullptr, *dv = nullptr, *dec = nullptr, *beta = nullptr, *dout = nullptr, *mw = nullptr, *msum = nullptr, *po = nullptr, *pml = nullptr, *ret_u = nullptr, *sgate = nullptr;
  int32_t *midx = nullptr, *mpos = nullptr, *mrb = nullptr;
  int moe_cap = 0;
  int4* chunk = nullptr;
  int32_t *row_seg = nullptr, *row_j = nullptr, *seg = nullptr, *nseg = nullptr, *state_len = nullptr, *parity = nullptr, *claim = nullptr, *err = nullptr, *head_rb = nullptr;
  // copies of whole groups
  float** st_bases = nullptr; int64_t* st_per = nullptr; int st_n = 0;
  char** pg_pools = nullptr; int64_t* pg_bytes = nullptr; int pg_n = 0;
  float* tap = nullptr; size_t tap_floats = 0;   // residual after every layer, on request
};

static inline int up_to(int v, int m) { return (v + m - 1) / m * m; }
bool heads_mfma_sizes(int d, int maps, int dv, bool f32, int* dkp, int* dvp);
#define IXT_HEADS_SPLIT_BLOCKS 1024              // few rows: blocks that the keys of a launch are split into (four per CU)

// What surrounds a sublayer: the norms behind it and in front of the next one, its own hyper-connection and the next one's (nullptr: there is none), the
// token shift in front of the next one.  to_cat: the next thing is the start of a pass, which takes x as it is
struct Around { NormW post, pre; const float *hc, *hc_next; const float* mu = nullptr; float* shift = nullptr; bool to_cat = false; };
// A sublayer's output: slices t, or the weighted sum of a row's expert outputs among them (pos, wts, top); add, times addw, and bias, times fbias, join it.
// fresh: it takes the place of x
struct SubOut { Slices t, add; const float* addw; const int32_t* pos; const float* wts; int top; const float* bias = nullptr; float fbias = 1.0f; bool fresh = false; };
// x <- x + post(t), the next operand pre(x), or the same among streams (k_sub_norm); routed: its f32 copy too; single: every row is the only one of its group
template <typename T>
int hybrid_norm(ixt_ctx* c, const SubOut& o, const Around& ar, bool routed, int R, bool single, hipStream_t st);
// rows lrows[i] (or lrow0 + i), n of them, of the residual stream -> the model's norm -> the head's operand
template <typename T>
int hybrid_final_norm(ixt_ctx* c, int R, int n, const int32_t* lrows, int lrow0, hipStream_t st);
// attention of a layer over heads: projection t -> pages, and the operand of the output projection in m->act.  L: the layer, W: the one with its parameters
template <typename T>
int heads_attention(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, int R, bool decode, int len_hint, hipStream_t st);
// one token per row, attention beside retention or lightning attention (L.side), t: the projection of both.  Done where `done` comes back true
template <typename T>
int heads_beside_retention(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, int R, int len_hint, hipStream_t st, bool* done);
static inline RetArgs ret_args(const HybridModel* m, const HLayer& L, const Slices& t) {
  return RetArgs{L.rg, t, L.pow, m->seg, m->chunk, m->nseg, m->dq, m->dk, m->dv, m->ret_u, L.state, m->dout, m->eps};
}
static inline size_t ret_step_lds(const RetGeom& g) { return sizeof(float) * (2 * g.dp + g.dvp + 256 / (g.dvp / 4) * g.dvp); }
// retention (or lightning attention) of a layer: projection t -> the operand of the output projection in m->act
template <typename T>
int retention_mix(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, int R, int nseg_max, bool single, hipStream_t st);
// selective scan: the convolved inputs (the second projection's operand, m->act); the third projection's operand (m->scan_t); everything behind it
// (dt empty, single only: the third projection as well)
template <typename T>
int scan_conv(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& in, int R, hipStream_t st);
template <typename T>
int scan_rank(ixt_ctx* c, const HLayer& W, const Slices& low, int R, hipStream_t st);
template <typename T>
int scan_mix(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& in, const Slices& low, const Slices& dt, int R, int nseg_max, bool single, hipStream_t st);
