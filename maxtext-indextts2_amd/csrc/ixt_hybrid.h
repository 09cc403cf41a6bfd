// ixt_hybrid.h -- what the host objects of hybrid decoders share: the model, its layer plans, and the launch helpers that live in objects of their own
// (they compile side by side): norms between sublayers (ixt_hybrid_norm.hip), attention over heads (ixt_hybrid_heads.hip).
#pragma once
#include "ixt_internal.h"
#include "ixt_heads_kernels.h"
#include "ixt_hybrid_kernels.h"
#include "ixt_retention_kernels.h"

struct HMat { void* w = nullptr; int K = 0, N = 0, Kp = 0, Np = 0; };       // a dot operand of the ctx's storage type, zero-padded
struct HLayer {
  ixt_layer c{};
  int src = 0;                                   // the layer whose parameters are used
  LatentGeom lg{};
  DeltaGeom dg{};
  HeadsGeom hg{};
  RetGeom rg{};
  HMat in, low, o, gu, down;                     // input projection, second low-rank product, output projection, gate | up (or up), down
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
  const float *rope_cos = nullptr, *rope_sin = nullptr;
  void* pages = nullptr;                         // latent layer: [page][token][rankp + rotp]; attention layer: keys [page][kv head][token][dkp]
  void* vpages = nullptr;                        // attention layer: values [page][kv head][token][dvp]
  float *state = nullptr, *tails = nullptr;      // delta layer: [group][H][dv][dp], [group][2][taps - 1][C]; retention: [group][H][dp][dvp]
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
  // workspaces
  float *x = nullptr, *part2 = nullptr, *h32 = nullptr;      // h32: a routed layer's normed input in f32
  size_t part2_floats = 0;
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

// What surrounds a sublayer: the norms behind it and in front of the next one, its own hyper-connection and the next one's (nullptr: there is none)
struct Around { NormW post, pre; const float *hc, *hc_next; };
// A sublayer's output: slices t, or the weighted sum of a row's expert outputs among them (pos, wts, top); add, times addw, joins it
struct SubOut { Slices t, add; const float* addw; const int32_t* pos; const float* wts; int top; };
// x <- x + post(t), the next operand pre(x), or the same among streams (k_sub_norm); routed: its f32 copy too
template <typename T>
int hybrid_norm(ixt_ctx* c, const SubOut& o, const Around& ar, bool routed, int R, hipStream_t st);
// rows lrows[i] (or lrow0 + i), n of them, of the residual stream -> the model's norm -> the head's operand
template <typename T>
int hybrid_final_norm(ixt_ctx* c, int R, int n, const int32_t* lrows, int lrow0, hipStream_t st);
// attention of a layer over heads: projection t -> pages, and the operand of the output projection in m->act.  L: the layer, W: the one with its parameters
template <typename T>
int heads_attention(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, int R, bool decode, int len_hint, hipStream_t st);
