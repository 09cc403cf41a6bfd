// ixt_hybrid.hip -- host side of IXT_BLOCK_HYBRID: layer plans, weight loading, caches and states, and the forward pass over rows that every engine
// entry point (prefill chunk, packed rows, decode step) ends in.
#include "ixt_internal.h"
#include "ixt_heads_kernels.h"
#include "ixt_hybrid_kernels.h"

struct HMat { void* w = nullptr; int K = 0, N = 0, Kp = 0, Np = 0; };       // a dot operand of the ctx's storage type, zero-padded
struct HLayer {
  ixt_layer c{};
  int src = 0;                                   // the layer whose parameters are used
  LatentGeom lg{};
  DeltaGeom dg{};
  HeadsGeom hg{};
  HMat in, low, o, gu, down;                     // input projection, second low-rank product, output projection, gate | up, down
  HMat uk, uv;                                   // per-head matrices of a latent layer (heads * wstride elements apart): d -> rank, rank -> v
  int d_off = 0;                                 // latent layer: column of the latent in the input projection
  size_t uk_stride = 0, uv_stride = 0, gu_stride = 0, down_stride = 0;
  NormW n1{}, n1b{}, n2{}, n2b{};                // in front of / behind the mixer, in front of / behind the feed-forward
  HMat sgu, sdown;                               // a mixture's shared unit
  float *qn = nullptr, *kn = nullptr, *sink = nullptr, *corr = nullptr;
  float *cnorm = nullptr, *cq = nullptr, *ck = nullptr, *cv = nullptr, *a_log = nullptr, *dt_bias = nullptr, *onorm = nullptr, *router = nullptr;
  const float *rope_cos = nullptr, *rope_sin = nullptr;
  void* pages = nullptr;                         // latent layer: [page][token][rankp + rotp]; attention layer: keys [page][kv head][token][dkp]
  void* vpages = nullptr;                        // attention layer: values [page][kv head][token][dvp]
  float *state = nullptr, *tails = nullptr;      // delta layer: [group][H][dv][dp], [group][2][taps - 1][C]
};
struct HTensor { std::vector<int64_t> shape; std::function<int(const void*, int, hipStream_t)> load; bool done = false; };   // load empty: accepted, unused
struct HybridModel {
  bool f32 = false, recurrent = false;
  size_t esz = 2;                                // bytes per activation / weight element
  int E = 0, Ep = 0, V = 0, maxH = 0, kmax_pad = 0, norm_kind = 0, norm_places = 0;      // maxH: most heads of a latent layer
  float emb_scale = 1.0f, eps = 1e-5f;
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
  float *dq = nullptr, *dk = nullptr, *dkq = nullptr, *dv = nullptr, *dec = nullptr, *beta = nullptr, *dout = nullptr, *mw = nullptr, *msum = nullptr, *po = nullptr, *pml = nullptr;
  int32_t *midx = nullptr, *mpos = nullptr, *mrb = nullptr;
  int moe_cap = 0;
  int32_t *row_seg = nullptr, *row_j = nullptr, *seg = nullptr, *nseg = nullptr, *state_len = nullptr, *parity = nullptr, *claim = nullptr, *err = nullptr, *head_rb = nullptr;
  // copies of whole groups
  float** st_bases = nullptr; int64_t* st_per = nullptr; int st_n = 0;
  char** pg_pools = nullptr; int64_t* pg_bytes = nullptr; int pg_n = 0;
  float* tap = nullptr; size_t tap_floats = 0;   // residual after every layer, on request
};

static int up_to(int v, int m) { return (v + m - 1) / m * m; }
// what one latent row is padded to: the matrix-core kernel's sizes, beyond them multiples of 32 (k_latent_attn_any)
static int latent_rankp(int rank) { return rank <= 64 ? 64 : rank <= 128 ? 128 : rank <= 256 ? 256 : rank <= 512 ? 512 : up_to(rank, 32); }
static int latent_rotp(int rot) { return rot <= 32 ? 32 : rot <= 64 ? 64 : up_to(rot, 32); }
// k_heads_prompt / k_heads_decode: the padded (key, value) sizes they are built for, cheapest first; none fits: k_heads_any
#define IXT_HEADS_SIZES(X) X(32, 32) X(64, 64) X(64, 128) X(128, 64) X(96, 96) X(128, 128) X(192, 128) X(192, 192) X(256, 256)
#define IXT_HEADS_SPLIT_BLOCKS 1024              // few rows: blocks that the keys of a launch are split into (four per CU)
static bool heads_mfma_sizes(int d, int dv, bool f32, int* dkp, int* dvp) {
  if (f32) return false;
#define X(DK_, DV_) if (d <= DK_ && dv <= DV_) { *dkp = DK_; *dvp = DV_; return true; }
  IXT_HEADS_SIZES(X)
#undef X
  return false;
}
static bool latent_mfma_fits(const HybridModel& m, const LatentGeom& g) { return !m.f32 && g.rankp <= 512 && g.rotp <= 64; }

static int h_alloc(ixt_ctx* c, void** p, size_t bytes) {      // zero-filled: padding behind real columns is never written and must read as zero
  char* q = nullptr;
  TRY(dmalloc(c, &q, bytes));
  HIPCHK(hipMemset(q, 0, bytes));
  *p = q;
  return IXT_OK;
}
template <typename P> static int h_allocf(ixt_ctx* c, P** p, size_t n) { return h_alloc(c, (void**)p, n * sizeof(P)); }
static int h_mat(ixt_ctx* c, HMat* m, int K, int N, size_t copies = 1) {
  m->K = K; m->N = N; m->Kp = up_to(K, IXT_KALIGN); m->Np = up_to(N, 16);
  return h_alloc(c, &m->w, (size_t)m->Kp * m->Np * copies * c->hy->esz);
}
// where `k_load_nk` puts a matrix of n columns and k inputs; the other fields of LoadMap by name
static LoadMap load_map(int n, int k, int Kp, int n_off = 0, int k_off = 0) {
  LoadMap m{};
  m.n = n; m.k = k; m.ld = k; m.Kp = Kp; m.n_off = n_off; m.k_off = k_off;
  return m;
}
template <typename T>
static int h_load_nk(const void* src, int dtype, T* dst, const LoadMap& lm, hipStream_t st) {
  const unsigned blocks = (unsigned)(((int64_t)lm.n * lm.k + 255) / 256);
  if (dtype == IXT_BF16) hipLaunchKernelGGL((k_load_nk<bf16_t, T>), dim3(blocks), dim3(256), 0, st, (const bf16_t*)src, dst, lm);
  else if (dtype == IXT_F32) hipLaunchKernelGGL((k_load_nk<float, T>), dim3(blocks), dim3(256), 0, st, (const float*)src, dst, lm);
  else return set_err(IXT_ERR_INVALID, "dtype %d", dtype);
  LAUNCHCHK();
  return IXT_OK;
}
template <typename T>
static int h_load_vec(const void* src, int dtype, T* dst, int64_t n, hipStream_t st) {
  const unsigned blocks = (unsigned)((n + 255) / 256);
  if (dtype == IXT_BF16) hipLaunchKernelGGL((k_load_vec<bf16_t, T>), dim3(blocks), dim3(256), 0, st, (const bf16_t*)src, dst, n);
  else if (dtype == IXT_F32) hipLaunchKernelGGL((k_load_vec<float, T>), dim3(blocks), dim3(256), 0, st, (const float*)src, dst, n);
  else return set_err(IXT_ERR_INVALID, "dtype %d", dtype);
  LAUNCHCHK();
  return IXT_OK;
}
static int h_load_mat(const HybridModel* m, const void* src, int dtype, void* dst, const LoadMap& lm, hipStream_t st) {
  return m->f32 ? h_load_nk(src, dtype, (float*)dst, lm, st) : h_load_nk(src, dtype, (bf16_t*)dst, lm, st);
}

int hybrid_check(const ixt_config& c) {
  if (!c.layers || c.num_decoder_layers < 1) return set_err(IXT_ERR_INVALID, "hybrid decoder: no layers");
  if (c.emb_dim < 1 || c.emb_dim > 12288 || c.vocab_size < 1) return set_err(IXT_ERR_UNSUPPORTED, "hybrid decoder: emb_dim %d (1 .. 12288), vocab_size %d", c.emb_dim, c.vocab_size);
  if (c.fp8_weights) return set_err(IXT_ERR_UNSUPPORTED, "hybrid decoder: fp8 weights are not built");
  if ((c.norm_kind != IXT_NORM_RMS && c.norm_kind != IXT_NORM_TANH) || c.norm_places < IXT_NORM_BEFORE || c.norm_places > (IXT_NORM_BEFORE | IXT_NORM_AFTER))
    return set_err(IXT_ERR_UNSUPPORTED, "hybrid decoder: norm kind %d, places %d", c.norm_kind, c.norm_places);
  for (int i = 0; i < c.num_decoder_layers; ++i) {
    const ixt_layer& l = c.layers[i];
    if (l.weights_of >= c.num_decoder_layers || (l.weights_of >= 0 && c.layers[l.weights_of].weights_of >= 0) || l.weights_of == i)
      return set_err(IXT_ERR_INVALID, "layer %d: weights_of %d", i, l.weights_of);
    if (l.heads < 1 || l.dim < 1 || l.vdim < 1) return set_err(IXT_ERR_INVALID, "layer %d: heads / dim / vdim", i);
    if (l.mixer == IXT_MIX_LATENT_ATTENTION) {
      if (l.kv_rank < 1 || l.kv_rank > 1024 || l.rot_dim < 0 || l.rot_dim % 2) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: kv_rank %d (1 .. 1024), rot_dim %d (even)", i, l.kv_rank, l.rot_dim);
    } else if (l.mixer == IXT_MIX_GATED_DELTA) {
      if (l.kv_heads < 1 || l.heads % l.kv_heads || l.conv < 1 || l.decay_rank < 1 || l.gate_rank < 1) return set_err(IXT_ERR_INVALID, "layer %d: kv_heads / conv / ranks", i);
      if (l.dim > 512) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: delta rule key dims %d (at most 512)", i, l.dim);
    } else if (l.mixer == IXT_MIX_ATTENTION) {
      if (l.kv_heads < 1 || l.heads % l.kv_heads || l.rot_dim < 0 || l.rot_dim % 2 || l.rot_dim > l.dim) return set_err(IXT_ERR_INVALID, "layer %d: kv_heads / rot_dim", i);
      if (l.dim > 4096 || l.vdim > 1024) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: %d key dims (at most 4096), %d value dims (at most 1024)", i, l.dim, l.vdim);
      if (!(l.attn_scale > 0.0f)) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: score factor %g (positive)", i, l.attn_scale);
      if (l.rope_factor > 0.0f && !(l.rope_low > 0.0f && l.rope_high > l.rope_low && l.rope_original > 0.0f)) return set_err(IXT_ERR_INVALID, "layer %d: rotation scaling", i);
    } else return set_err(IXT_ERR_UNSUPPORTED, "layer %d: mixer %d", i, l.mixer);
    if (l.ffn != IXT_FFN_NONE && (l.glu < IXT_GLU_CLAMPED || l.glu > IXT_GLU_SILU)) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: gated unit %d", i, l.glu);
    if (l.ffn == IXT_FFN_MOE) {
      if (l.experts < 1 || l.experts > 1024 || l.top < 1 || l.top > l.experts || l.ff < 1 || l.shared_ff < 0)
        return set_err(IXT_ERR_UNSUPPORTED, "layer %d: experts %d (1 .. 1024), top %d", i, l.experts, l.top);
      if (l.router != IXT_ROUTE_SOFTMAX && l.router != IXT_ROUTE_SIGMOID) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: router %d", i, l.router);
      if (l.groups > 1 && (l.experts % l.groups || l.groups_keep < 1 || l.groups_keep > l.groups || l.top > l.experts / l.groups * l.groups_keep))
        return set_err(IXT_ERR_INVALID, "layer %d: %d of %d groups of experts, top %d", i, l.groups_keep, l.groups, l.top);
    } else if (l.ffn == IXT_FFN_DENSE) {
      if (l.ff < 1) return set_err(IXT_ERR_INVALID, "layer %d: ff", i);
    } else if (l.ffn != IXT_FFN_NONE) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: ffn %d", i, l.ffn);
  }
  return IXT_OK;
}

// a norm's tensors: `name`, and for a tanh norm name.alpha (a scalar) and name.b; zeros behind the E features
static int hybrid_norm_params(ixt_ctx* c, const std::string& name, NormW* w) {
  HybridModel* m = c->hy;
  const int E = m->E;
  auto one = [&](const std::string& t, const float** dst, int64_t n, std::vector<int64_t> shape) -> int {
    float* d = nullptr;
    TRY(h_allocf(c, &d, (size_t)m->Ep));
    *dst = d;
    m->tensors[t] = HTensor{std::move(shape), [=](const void* s, int dt, hipStream_t st) { return h_load_vec(s, dt, d, n, st); }, false};
    return IXT_OK;
  };
  TRY(one(name, &w->w, E, {E}));
  if (m->norm_kind == IXT_NORM_TANH) {
    TRY(one(name + ".alpha", &w->alpha, 1, {}));
    TRY(one(name + ".b", &w->b, E, {E}));
  }
  return IXT_OK;
}

// parameters of layer i (its own tensors; a layer with weights_of has none)
static int hybrid_layer_params(ixt_ctx* c, int i) {
  HybridModel* m = c->hy;
  HLayer& L = m->layers[i];
  const ixt_layer& l = L.c;
  const int E = m->E;
  const std::string p = "l" + std::to_string(i) + ".";
  auto add = [&](const std::string& name, std::vector<int64_t> shape, std::function<int(const void*, int, hipStream_t)> f) { m->tensors[p + name] = HTensor{std::move(shape), std::move(f), false}; };
  auto vec = [&](const std::string& name, float** dst, int64_t n, std::vector<int64_t> shape) -> int {
    TRY(h_allocf(c, dst, (size_t)up_to((int)n, 4)));
    float* d = *dst;
    add(name, std::move(shape), [d, n](const void* s, int dt, hipStream_t st) { return h_load_vec(s, dt, d, n, st); });
    return IXT_OK;
  };
  auto mat_as = [&](const std::string& name, const HMat& M, const LoadMap& lm, size_t elem_off = 0) {
    char* d = (char*)M.w + elem_off * m->esz;
    add(name, {lm.n, lm.k}, [=](const void* s, int dt, hipStream_t st) { return h_load_mat(m, s, dt, d, lm, st); });
  };
  auto mat = [&](const std::string& name, const HMat& M, int n, int k, int n_off, int k_off = 0) { mat_as(name, M, load_map(n, k, M.Kp, n_off, k_off)); };
  auto norm = [&](const std::string& name, NormW* w) -> int { return hybrid_norm_params(c, p + name, w); };
  const bool both = m->norm_places == (IXT_NORM_BEFORE | IXT_NORM_AFTER);
  TRY(norm("norm1", m->norm_places & IXT_NORM_BEFORE ? &L.n1 : &L.n1b));
  if (both) TRY(norm("norm1b", &L.n1b));
  if (l.mixer == IXT_MIX_LATENT_ATTENTION) {
    const LatentGeom& g = L.lg;
    const int NQ = g.H * (g.dn + g.dr);
    TRY(h_mat(c, &L.in, E, L.d_off + g.rank + g.dr));
    mat("mix.q", L.in, NQ, E, 0);
    mat("mix.dkv", L.in, g.rank + g.dr, E, L.d_off);
    TRY(vec("mix.dkv.norm", &L.cnorm, g.rank, {g.rank}));
    TRY(h_mat(c, &L.uk, g.dn, g.rankp, g.H));
    TRY(h_mat(c, &L.uv, g.rankp, l.vdim, g.H));
    L.uk_stride = (size_t)L.uk.Kp * L.uk.Np; L.uv_stride = (size_t)L.uv.Kp * L.uv.Np;
    const HLayer* Lp = &L;
    add("mix.uk", {(int64_t)g.H * g.dn, g.rank}, [=](const void* s, int dt, hipStream_t st) {     // [h dn + i][c] -> per head (k = i, n = c): queries into latent space
      LoadMap uk = load_map(Lp->lg.rank, Lp->lg.dn, Lp->uk.Kp);
      uk.trans = 1; uk.ld = uk.n;
      for (int h = 0; h < Lp->lg.H; ++h)
        TRY(h_load_mat(m, (const char*)s + (size_t)h * Lp->lg.dn * Lp->lg.rank * (dt == IXT_F32 ? 4 : 2), dt, (char*)Lp->uk.w + h * Lp->uk_stride * m->esz, uk, st));
      return (int)IXT_OK;
    });
    add("mix.uv", {(int64_t)g.H * l.vdim, g.rank}, [=](const void* s, int dt, hipStream_t st) {
      for (int h = 0; h < Lp->lg.H; ++h)
        TRY(h_load_mat(m, (const char*)s + (size_t)h * Lp->c.vdim * Lp->lg.rank * (dt == IXT_F32 ? 4 : 2), dt, (char*)Lp->uv.w + h * Lp->uv_stride * m->esz, load_map(Lp->c.vdim, Lp->lg.rank, Lp->uv.Kp), st));
      return (int)IXT_OK;
    });
    TRY(h_mat(c, &L.o, g.H * l.vdim, E));
    mat("mix.o", L.o, E, g.H * l.vdim, 0);
  } else if (l.mixer == IXT_MIX_ATTENTION) {
    const HeadsGeom& g = L.hg;
    TRY(h_mat(c, &L.in, E, g.ov + g.G * g.vs));
    LoadMap q = load_map(g.H * g.d, E, L.in.Kp), k = load_map(g.G * g.d, E, L.in.Kp, g.ok), v = load_map(g.G * g.dv, E, L.in.Kp, g.ov);
    q.ng = k.ng = g.d; q.ngp = k.ngp = g.hs; v.ng = g.dv; v.ngp = g.vs;
    mat_as("mix.q", L.in, q);
    mat_as("mix.k", L.in, k);
    mat_as("mix.v", L.in, v);
    if (l.qk_norm) { TRY(vec("mix.q.norm", &L.qn, g.d, {g.d})); TRY(vec("mix.k.norm", &L.kn, g.d, {g.d})); }
    if (l.sink) TRY(vec("mix.sink", &L.sink, g.H, {g.H}));
    TRY(h_mat(c, &L.o, g.H * g.vs, E));
    LoadMap o = load_map(E, g.H * g.dv, L.o.Kp);
    o.kg = g.dv; o.kgp = g.vs;
    mat_as("mix.o", L.o, o);
  } else {
    const DeltaGeom& g = L.dg;
    TRY(h_mat(c, &L.in, E, g.og + g.rg));
    mat("mix.q", L.in, g.KH * g.d, E, g.oq);
    mat("mix.k", L.in, g.KH * g.d, E, g.ok);
    mat("mix.v", L.in, g.H * g.dv, E, g.ov);
    mat("mix.b", L.in, g.H, E, g.ob);
    mat("mix.a1", L.in, g.ra, E, g.oa);
    mat("mix.g1", L.in, g.rg, E, g.og);
    TRY(h_mat(c, &L.low, g.ra + g.rg, g.og2 + g.H * g.dv));
    mat("mix.a2", L.low, g.H * g.d, g.ra, 0, 0);
    mat("mix.g2", L.low, g.H * g.dv, g.rg, g.og2, g.ra);
    TRY(vec("mix.q.conv", &L.cq, (int64_t)g.KH * g.d * g.taps, {g.KH * g.d, g.taps}));
    TRY(vec("mix.k.conv", &L.ck, (int64_t)g.KH * g.d * g.taps, {g.KH * g.d, g.taps}));
    TRY(vec("mix.v.conv", &L.cv, (int64_t)g.H * g.dv * g.taps, {g.H * g.dv, g.taps}));
    TRY(vec("mix.A_log", &L.a_log, g.H, {g.H}));
    TRY(vec("mix.dt_bias", &L.dt_bias, (int64_t)g.H * g.d, {g.H * g.d}));
    TRY(vec("mix.norm", &L.onorm, g.dv, {g.dv}));
    TRY(h_mat(c, &L.o, g.H * g.dv, E));
    mat("mix.o", L.o, E, g.H * g.dv, 0);
  }
  if (l.ffn == IXT_FFN_NONE) {                                   // a layer without a feed-forward has no use for its norms
    for (const char* n : {"norm2", "norm2b"}) {
      if (!both && std::string(n) == "norm2b") continue;
      m->tensors[p + n] = HTensor{{E}, nullptr, true};
      if (m->norm_kind == IXT_NORM_TANH) { m->tensors[p + n + ".alpha"] = HTensor{{}, nullptr, true}; m->tensors[p + n + ".b"] = HTensor{{E}, nullptr, true}; }
    }
    return IXT_OK;
  }
  TRY(norm("norm2", m->norm_places & IXT_NORM_BEFORE ? &L.n2 : &L.n2b));
  if (both) TRY(norm("norm2b", &L.n2b));
  auto unit = [&](const std::string& q, const HMat& gu, const HMat& down, int ff, size_t gu_off = 0, size_t down_off = 0) {
    LoadMap gate = load_map(ff, E, gu.Kp), up = load_map(ff, E, gu.Kp, 1);
    gate.inter = up.inter = 1;
    mat_as(q + "gate", gu, gate, gu_off);
    mat_as(q + "up", gu, up, gu_off);
    mat_as(q + "down", down, load_map(E, ff, down.Kp), down_off);
  };
  const bool moe = l.ffn == IXT_FFN_MOE;
  const int n = moe ? l.experts : 1;
  TRY(h_mat(c, &L.gu, E, 2 * up_to(l.ff, IXT_KALIGN), n));
  TRY(h_mat(c, &L.down, l.ff, E, n));
  L.gu_stride = (size_t)L.gu.Kp * L.gu.Np; L.down_stride = (size_t)L.down.Kp * L.down.Np;
  for (int e = 0; e < n; ++e) unit(moe ? "mlp.e" + std::to_string(e) + "." : "mlp.", L.gu, L.down, l.ff, e * L.gu_stride, e * L.down_stride);
  if (!moe) return IXT_OK;
  if (l.shared_ff > 0) {
    TRY(h_mat(c, &L.sgu, E, 2 * up_to(l.shared_ff, IXT_KALIGN)));
    TRY(h_mat(c, &L.sdown, l.shared_ff, E));
    unit("mlp.shared.", L.sgu, L.sdown, l.shared_ff);
  }
  TRY(h_allocf(c, &L.router, (size_t)l.experts * m->Ep));
  float* d = L.router;
  const LoadMap lm = load_map(l.experts, E, m->Ep);
  add("mlp.router", {l.experts, E}, [=](const void* s, int dt, hipStream_t st) { return h_load_nk(s, dt, d, lm, st); });
  if (l.router_correction) TRY(vec("mlp.correction", &L.corr, l.experts, {l.experts}));
  return IXT_OK;
}

// rotation tables of a layer, f32 [position][rot_dim / 2] cos and sin of angles in f64; layers with the same rotation share them
static int hybrid_rope(ixt_ctx* c, const ixt_layer& l, std::map<std::vector<float>, std::pair<float*, float*>>* ropes, HLayer* L) {
  const std::vector<float> key = {(float)l.rot_dim, l.rope_base, l.rope_factor, l.rope_low, l.rope_high, l.rope_original};
  auto it = ropes->find(key);
  if (it == ropes->end()) {
    const int half = l.rot_dim / 2;
    std::vector<float> cs((size_t)c->Tmax * half + 1), sn((size_t)c->Tmax * half + 1);
    for (int j = 0; j < half; ++j) {
      double f = pow((double)l.rope_base, -2.0 * j / l.rot_dim);
      if (l.rope_factor > 0.0f) {
        const double turns = l.rope_original * f / (2.0 * M_PI);            // of this pair over the original context
        if (turns < l.rope_low) f /= l.rope_factor;
        else if (turns <= l.rope_high) { const double s = (turns - l.rope_low) / ((double)l.rope_high - l.rope_low); f = (1.0 - s) * f / l.rope_factor + s * f; }
      }
      for (int p = 0; p < c->Tmax; ++p) { cs[(size_t)p * half + j] = (float)cos(p * f); sn[(size_t)p * half + j] = (float)sin(p * f); }
    }
    float *dc = nullptr, *ds = nullptr;
    TRY(h_allocf(c, &dc, cs.size())); TRY(h_allocf(c, &ds, sn.size()));
    HIPCHK(hipMemcpy(dc, cs.data(), cs.size() * 4, hipMemcpyHostToDevice));
    HIPCHK(hipMemcpy(ds, sn.data(), sn.size() * 4, hipMemcpyHostToDevice));
    it = ropes->emplace(key, std::make_pair(dc, ds)).first;
  }
  L->rope_cos = it->second.first; L->rope_sin = it->second.second;
  return IXT_OK;
}

// everything a hybrid ctx owns besides the page state and the row descriptors (which all contexts share)
int hybrid_init(ixt_ctx* c) {
  const ixt_config& cf = c->cfg;
  HybridModel* m = c->hy;
  m->f32 = cf.float32 != 0; m->esz = m->f32 ? 4 : 2;
  m->E = cf.emb_dim; m->Ep = up_to(m->E, IXT_KALIGN); m->V = cf.vocab_size; m->emb_scale = cf.embedding_scale; m->eps = cf.normalization_layer_epsilon;
  m->norm_kind = cf.norm_kind; m->norm_places = cf.norm_places;
  const int n = cf.num_decoder_layers, R = c->Rmax, Rp = up_to(R, 128);
  m->layers.resize(n);
  TRY(h_alloc(c, &m->embed, (size_t)m->V * m->E * m->esz));
  { void* d = m->embed; const int64_t ne = (int64_t)m->V * m->E; const bool f = m->f32;
    m->tensors["embed"] = HTensor{{m->V, m->E}, [=](const void* s, int dt, hipStream_t st) { return f ? h_load_vec(s, dt, (float*)d, ne, st) : h_load_vec(s, dt, (bf16_t*)d, ne, st); }, false}; }
  TRY(h_mat(c, &m->head, m->E, m->V));
  { void* d = m->head.w; const LoadMap lm = load_map(m->V, m->E, m->head.Kp);
    m->tensors["head"] = HTensor{{m->V, m->E}, [=](const void* s, int dt, hipStream_t st) { return h_load_mat(m, s, dt, d, lm, st); }, false}; }
  TRY(hybrid_norm_params(c, "final.norm", &m->fnorm));
  std::map<std::vector<float>, std::pair<float*, float*>> ropes;
  size_t act_k = m->Ep, hact_k = 0, qx_e = 0, qr_e = 0, olat_e = 0, part = 0, part2 = 0, s_q = 0, s_kq = 0, s_v = 0, s_dec = 0, s_b = 0, xg_e = 0, mh_e = 0, mi = 0, po = 0;
  auto upd = [](size_t& a, size_t v) { if (v > a) a = v; };
  // f32 slices of a dot over at most R rows (split-K only below 128 rows; launch_dot keeps to one slice when the slices do not fit)
  auto dotsz = [&](int K, int N) { upd(part, std::max((size_t)R * N, (size_t)std::min(R, 128) * N * ((K + IXT_CHAIN - 1) / IXT_CHAIN))); };
  for (int i = 0; i < n; ++i) {
    HLayer& L = m->layers[i];
    L.c = cf.layers[i];
    L.src = L.c.weights_of >= 0 ? L.c.weights_of : i;
    const ixt_layer& l = L.c;
    if (l.mixer == IXT_MIX_LATENT_ATTENTION) {
      LatentGeom& g = L.lg;
      g.H = l.heads; g.dn = l.dim; g.dr = l.rot_dim; g.rank = l.kv_rank; g.P = c->P; g.mpg = c->mpg; g.window = l.window; g.scale = l.attn_scale;
      g.rankp = latent_rankp(l.kv_rank); g.rotp = latent_rotp(l.rot_dim);
      L.d_off = up_to(g.H * (g.dn + g.dr), 16);
      TRY(h_alloc(c, &L.pages, (size_t)cf.pagedattn_num_pages * c->P * (g.rankp + g.rotp) * m->esz));
      TRY(hybrid_rope(c, l, &ropes, &L));
      m->maxH = std::max(m->maxH, g.H);
      const int dnp = up_to(g.dn, IXT_KALIGN), ukn = up_to(g.rankp, 16), kp = up_to(g.rankp, IXT_KALIGN), uvn = up_to(l.vdim, 16);
      dotsz(m->Ep, up_to(L.d_off + g.rank + g.dr, 16));
      upd(part, (size_t)g.H * Rp * ukn);                                    // several slices only below 128 rows
      upd(part, (size_t)g.H * up_to(std::min(R, 128), 16) * ukn * ((dnp + IXT_CHAIN - 1) / IXT_CHAIN));
      upd(part, (size_t)g.H * Rp * uvn);
      upd(part, (size_t)g.H * up_to(std::min(R, 128), 16) * uvn * ((kp + IXT_CHAIN - 1) / IXT_CHAIN));
      dotsz(up_to(g.H * l.vdim, IXT_KALIGN), up_to(m->E, 16));
      upd(act_k, up_to(g.H * l.vdim, IXT_KALIGN));
      upd(qx_e, (size_t)g.H * Rp * dnp); upd(qr_e, (size_t)R * g.H * g.rotp); upd(olat_e, (size_t)g.H * Rp * kp);
      upd(po, (size_t)(1024 + g.H) * 16 * g.rankp);
    } else if (l.mixer == IXT_MIX_ATTENTION) {
      HeadsGeom& g = L.hg;
      g.H = l.heads; g.G = l.kv_heads; g.d = l.dim; g.dv = l.vdim; g.rot = l.rot_dim; g.P = c->P; g.mpg = c->mpg; g.window = l.window; g.scale = l.attn_scale;
      if (!heads_mfma_sizes(l.dim, l.vdim, m->f32, &g.dkp, &g.dvp)) { g.dkp = up_to(l.dim, 32); g.dvp = up_to(l.vdim, 32); }
      g.hs = up_to(l.dim, 4); g.vs = up_to(l.vdim, 4); g.ok = up_to(g.H * g.hs, 16); g.ov = g.ok + up_to(g.G * g.hs, 16);
      const size_t tokens = (size_t)cf.pagedattn_num_pages * c->P * g.G;
      if (tokens > (size_t)INT32_MAX) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: %zu cached heads in the page pool", i, tokens);
      TRY(h_alloc(c, &L.pages, tokens * g.dkp * m->esz));
      TRY(h_alloc(c, &L.vpages, tokens * g.dvp * m->esz));
      TRY(hybrid_rope(c, l, &ropes, &L));
      dotsz(m->Ep, up_to(g.ov + g.G * g.vs, 16));
      dotsz(up_to(g.H * g.vs, IXT_KALIGN), up_to(m->E, 16));
      upd(act_k, up_to(g.H * g.vs, IXT_KALIGN));
      upd(qx_e, (size_t)R * g.H * g.dkp);
      upd(po, (size_t)IXT_HEADS_SPLIT_BLOCKS * 16 * g.dvp);
    } else {
      m->recurrent = true;
      DeltaGeom& g = L.dg;
      g.H = l.heads; g.KH = l.kv_heads; g.d = l.dim; g.dv = l.vdim; g.taps = l.conv; g.ra = l.decay_rank; g.rg = l.gate_rank;
      int rp = 1;
      while (16 * rp < g.d) rp *= 2;
      g.dp = 16 * rp;
      g.oq = 0; g.ok = up_to(g.KH * g.d, 16); g.ov = g.ok + up_to(g.KH * g.d, 16); g.ob = g.ov + up_to(g.H * g.dv, 16);
      g.oa = g.ob + up_to(g.H, 16); g.og = g.oa + up_to(g.ra, 16); g.og2 = up_to(g.H * g.d, 16); g.C = 2 * g.KH * g.d + g.H * g.dv;
      TRY(h_allocf(c, &L.state, (size_t)c->G * g.H * g.dv * g.dp));
      TRY(h_allocf(c, &L.tails, (size_t)c->G * 2 * (g.taps - 1) * g.C + 4));
      dotsz(m->Ep, up_to(g.og + g.rg, 16));
      { const int K = up_to(g.ra + g.rg, IXT_KALIGN), N = up_to(g.og2 + g.H * g.dv, 16); upd(part2, std::max((size_t)R * N, (size_t)std::min(R, 128) * N * ((K + IXT_CHAIN - 1) / IXT_CHAIN))); }
      dotsz(up_to(g.H * g.dv, IXT_KALIGN), up_to(m->E, 16));
      upd(act_k, up_to(g.ra + g.rg, IXT_KALIGN)); upd(act_k, up_to(g.H * g.dv, IXT_KALIGN));
      upd(s_q, (size_t)R * g.KH * g.dp); upd(s_kq, (size_t)R * g.KH); upd(s_v, (size_t)R * g.H * g.dv); upd(s_dec, (size_t)R * g.H * g.dp); upd(s_b, (size_t)R * g.H);
    }
    if (l.ffn == IXT_FFN_DENSE) {
      const int Fp = up_to(l.ff, IXT_KALIGN);
      upd(hact_k, Fp);
      if (m->f32) upd(part, (size_t)R * 2 * Fp);
      dotsz(Fp, up_to(m->E, 16));
    } else if (l.ffn == IXT_FFN_MOE) {
      const int Fp = up_to(l.ff, IXT_KALIGN);
      if ((int64_t)R * l.top > (1 << 24)) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: %d rows x %d experts per token: smaller max_packed_rows / max_prefill_predict_length", i, R, l.top);
      const int pairs = R * l.top, cap = std::max(up_to(pairs, 128) + 128 * std::min(l.experts, pairs), 64 + 16 * l.experts);
      m->moe_cap = std::max(m->moe_cap, cap);
      upd(xg_e, (size_t)cap * m->Ep); upd(mh_e, (size_t)cap * Fp); upd(mi, (size_t)pairs);
      upd(part, (size_t)cap * up_to(m->E, 16));
      upd(part, (size_t)(64 + 16 * std::min(l.experts, 64)) * up_to(m->E, 16) * ((Fp + IXT_CHAIN - 1) / IXT_CHAIN));
      if (m->f32) upd(part, (size_t)cap * 2 * Fp);
      if (l.shared_ff > 0) {
        const int Sp = up_to(l.shared_ff, IXT_KALIGN), N = up_to(m->E, 16);
        upd(hact_k, Sp);
        if (m->f32) upd(part, (size_t)R * 2 * Sp);
        upd(part2, std::max((size_t)R * N, (size_t)std::min(R, 128) * N * ((Sp + IXT_CHAIN - 1) / IXT_CHAIN)));
      }
      if (!m->h32 && (m->norm_places & IXT_NORM_BEFORE)) TRY(h_allocf(c, &m->h32, (size_t)R * m->E));
    }
  }
  for (int i = 0; i < n; ++i)
    if (m->layers[i].src == i) TRY(hybrid_layer_params(c, i));
  m->missing = 0;
  for (auto& kv : m->tensors) m->missing += kv.second.done ? 0 : 1;
  upd(part, (size_t)c->NLmax * m->head.Np * (c->NLmax < 128 ? (m->head.Kp + IXT_CHAIN - 1) / IXT_CHAIN : 1));
  c->part_floats = part; TRY(h_allocf(c, &c->part, part));
  m->part2_floats = part2; TRY(h_allocf(c, &m->part2, part2 + 4));
  TRY(h_allocf(c, &m->x, (size_t)R * m->E));
  TRY(h_alloc(c, &m->xb, (size_t)Rp * m->Ep * m->esz));
  TRY(h_alloc(c, &m->act, (size_t)Rp * act_k * m->esz));
  TRY(h_alloc(c, &m->hact, (size_t)Rp * (hact_k + 8) * m->esz));
  TRY(h_alloc(c, &m->xn, (size_t)up_to(c->NLmax, 128) * m->Ep * m->esz));
  TRY(h_alloc(c, &m->qx, (qx_e + 8) * m->esz)); TRY(h_alloc(c, &m->qr, (qr_e + 8) * m->esz)); TRY(h_alloc(c, &m->olat, (olat_e + 8) * m->esz));
  TRY(h_alloc(c, &m->xg, (xg_e + 8) * m->esz)); TRY(h_alloc(c, &m->mhact, (mh_e + 8) * m->esz));
  TRY(h_allocf(c, &m->dq, s_q + 4)); TRY(h_allocf(c, &m->dk, s_q + 4)); TRY(h_allocf(c, &m->dkq, s_kq + 4)); TRY(h_allocf(c, &m->dv, s_v + 4));
  TRY(h_allocf(c, &m->dec, s_dec + 4)); TRY(h_allocf(c, &m->beta, s_b + 4)); TRY(h_allocf(c, &m->dout, s_v + 4));
  TRY(h_allocf(c, &m->mw, mi + 4)); TRY(h_allocf(c, &m->midx, mi + 4)); TRY(h_allocf(c, &m->mpos, mi + 4));
  TRY(h_allocf(c, &m->mrb, (size_t)m->moe_cap / 16 + 16));
  TRY(h_allocf(c, &m->msum, (size_t)64 * up_to(m->E, 16)));
  TRY(h_allocf(c, &m->po, po + 4)); TRY(h_allocf(c, &m->pml, (size_t)(IXT_HEADS_SPLIT_BLOCKS + m->maxH) * 16 * 2 + 4));
  TRY(h_allocf(c, &m->row_seg, (size_t)R)); TRY(h_allocf(c, &m->row_j, (size_t)R)); TRY(h_allocf(c, &m->seg, (size_t)R * 8)); TRY(h_allocf(c, &m->nseg, 4));
  TRY(h_allocf(c, &m->state_len, (size_t)c->G)); TRY(h_allocf(c, &m->parity, (size_t)c->G)); TRY(h_allocf(c, &m->claim, (size_t)c->G)); TRY(h_allocf(c, &m->err, 4));
  TRY(h_allocf(c, &m->head_rb, (size_t)m->maxH * Rp / 16 + 16));
  c->amax_cap = (size_t)c->NLmax * ((m->V + 1023) / 1024);
  TRY(h_allocf(c, &c->amax_val, c->amax_cap)); TRY(h_allocf(c, &c->amax_idx, c->amax_cap));
  // what a copy of a whole page group moves
  std::vector<float*> sb; std::vector<int64_t> sp, pb; std::vector<char*> pp;
  for (HLayer& L : m->layers) {
    if (L.c.mixer == IXT_MIX_ATTENTION) {
      pp.push_back((char*)L.pages); pb.push_back((int64_t)c->P * L.hg.G * L.hg.dkp * (int64_t)m->esz);
      pp.push_back((char*)L.vpages); pb.push_back((int64_t)c->P * L.hg.G * L.hg.dvp * (int64_t)m->esz);
    } else if (L.c.mixer == IXT_MIX_LATENT_ATTENTION) { pp.push_back((char*)L.pages); pb.push_back((int64_t)c->P * (L.lg.rankp + L.lg.rotp) * (int64_t)m->esz); }
    else { sb.push_back(L.state); sp.push_back((int64_t)L.dg.H * L.dg.dv * L.dg.dp); sb.push_back(L.tails); sp.push_back((int64_t)2 * (L.dg.taps - 1) * L.dg.C); }
  }
  m->st_n = (int)sb.size(); m->pg_n = (int)pp.size();
  TRY(h_allocf(c, &m->st_bases, sb.size() + 1)); TRY(h_allocf(c, &m->st_per, sb.size() + 1)); TRY(h_allocf(c, &m->pg_pools, pp.size() + 1)); TRY(h_allocf(c, &m->pg_bytes, pp.size() + 1));
  if (!sb.empty()) { HIPCHK(hipMemcpy(m->st_bases, sb.data(), sb.size() * sizeof(float*), hipMemcpyHostToDevice)); HIPCHK(hipMemcpy(m->st_per, sp.data(), sp.size() * 8, hipMemcpyHostToDevice)); }
  if (!pp.empty()) { HIPCHK(hipMemcpy(m->pg_pools, pp.data(), pp.size() * sizeof(char*), hipMemcpyHostToDevice)); HIPCHK(hipMemcpy(m->pg_bytes, pb.data(), pb.size() * 8, hipMemcpyHostToDevice)); }
  return IXT_OK;
}

int hybrid_load_weight(ixt_ctx* c, const std::string& name, const void* src, int dtype, const int64_t* shape, int ndim, hipStream_t st) {
  HybridModel* m = c->hy;
  auto it = m->tensors.find(name);
  if (it == m->tensors.end()) return set_err(IXT_ERR_INVALID, "unknown parameter %s", name.c_str());
  HTensor& t = it->second;
  bool same = ndim == (int)t.shape.size();
  for (int i = 0; same && i < ndim; ++i) same = shape[i] == t.shape[i];
  if (t.shape.empty()) same = ndim == 0 || (ndim == 1 && shape[0] == 1);       // a scalar
  if (!same) {
    std::string want;
    for (int64_t v : t.shape) want += (want.empty() ? "" : " x ") + std::to_string(v);
    return set_err(IXT_ERR_INVALID, "%s: expected %s", name.c_str(), want.c_str());
  }
  if (t.load) TRY(t.load(src, dtype, st));
  if (!t.done) { t.done = true; --m->missing; }
  return IXT_OK;
}

// pages and state of group src -> group dst (dst's pages reserved for `length` tokens) / state only (the page list moves elsewhere)
int hybrid_copy_group(ixt_ctx* c, int src, int dst, int npages, hipStream_t st) {
  HybridModel* m = c->hy;
  if (npages > 0 && m->pg_n > 0) hipLaunchKernelGGL(k_latent_pages_copy, dim3(npages, m->pg_n), dim3(256), 0, st, c->ps, src, dst, m->pg_pools, m->pg_bytes, c->P);
  if (m->st_n > 0) hipLaunchKernelGGL(k_state_copy, dim3(256), dim3(256), 0, st, m->st_bases, m->st_per, m->st_n, src, dst, m->state_len, m->parity);
  LAUNCHCHK();
  return IXT_OK;
}

// ---------------------------------------------------------------------------------------------------- the forward pass
template <typename T> static int hdot(ixt_ctx* c, const T* x, const HMat& w, int R, float* out, size_t out_floats, hipStream_t st, Slices* res);
template <> int hdot<bf16_t>(ixt_ctx* c, const bf16_t* x, const HMat& w, int R, float* out, size_t out_floats, hipStream_t st, Slices* res) {
  if (R <= c->small_rows && (size_t)R * w.Np <= out_floats && w.Np <= 65536 && sdot_plan(c, GEPI_F32, false, w.Kp, w.Np, R).ok) {     // few rows: one slice
    GemmEpi e{};
    e.out = out;
    TRY(launch_sdot(c, GEPI_F32, false, x, nullptr, (const bf16_t*)w.w, w.Kp, w.Np, R, e, st));
    *res = Slices{out, 1, (size_t)R * w.Np, w.Np};
    return IXT_OK;
  }
  DotResult dr;
  TRY(launch_dot(c, x, (const bf16_t*)w.w, w.Kp, w.Np, R, out, out_floats, false, st, &dr));
  *res = Slices{out, dr.slices, dr.slice_stride, w.Np};
  return IXT_OK;
}
template <> int hdot<float>(ixt_ctx*, const float* x, const HMat& w, int R, float* out, size_t out_floats, hipStream_t st, Slices* res) {
  if ((size_t)R * w.Np > out_floats) return set_err(IXT_ERR_INVALID, "dot: output workspace too small");
  hipLaunchKernelGGL(k_dot32, dim3((w.Np + 63) / 64, (R + 15) / 16), dim3(256), 0, st, x, (const float*)w.w, w.Kp, w.Np, R, out, (const int32_t*)nullptr, (size_t)0);
  LAUNCHCHK();
  *res = Slices{out, 1, (size_t)R * w.Np, w.Np};
  return IXT_OK;
}
// rows of several groups (heads, experts): 16-row block b uses the matrix of group rb_exp[b], `stride` elements apart.  group_rows: what every group's
// rows are aligned to (128: the ring GEMM)
template <typename T> static int hdot_grouped(ixt_ctx* c, const T* x, const HMat& w, size_t stride, int rows, int group_rows, const int32_t* rb, float* out, size_t out_floats, hipStream_t st, Slices* res);
template <> int hdot_grouped<bf16_t>(ixt_ctx* c, const bf16_t* x, const HMat& w, size_t stride, int rows, int group_rows, const int32_t* rb, float* out, size_t out_floats, hipStream_t st, Slices* res) {
  if (group_rows % 128 == 0) {
    if ((size_t)rows * w.Np > out_floats) return set_err(IXT_ERR_INVALID, "grouped dot: output workspace too small");
    GemmEpi e{};
    e.out = out; e.rb_exp = rb; e.wstride = stride / 8;
    TRY(launch_ring(c, GEPI_F32, x, (const bf16_t*)w.w, w.Kp, w.Np, rows, e, false, st));
    *res = Slices{out, 1, (size_t)rows * w.Np, w.Np};
    return IXT_OK;
  }
  const int chains = (w.Kp + IXT_CHAIN - 1) / IXT_CHAIN, ntile = w.Np / 16, zblocks = (rows + 15) / 16;
  if ((size_t)chains * rows * w.Np > out_floats) return set_err(IXT_ERR_INVALID, "grouped dot: slice workspace too small");
  hipLaunchKernelGGL((k_dotb<1, true, true>), dim3((((ntile + 3) / 4 + 7) / 8) * 8 * zblocks, chains), dim3(256), (size_t)16 * 1024, st, reinterpret_cast<const u32x4*>(x),
                     reinterpret_cast<const u32x4*>(w.w), w.Kp, w.Np, rows, out, ntile, zblocks, rb, stride / 8, 0, 0.0f);
  LAUNCHCHK();
  *res = Slices{out, chains, (size_t)rows * w.Np, w.Np};
  return IXT_OK;
}
template <> int hdot_grouped<float>(ixt_ctx*, const float* x, const HMat& w, size_t stride, int rows, int, const int32_t* rb, float* out, size_t out_floats, hipStream_t st, Slices* res) {
  if ((size_t)rows * w.Np > out_floats) return set_err(IXT_ERR_INVALID, "grouped dot: output workspace too small");
  hipLaunchKernelGGL(k_dot32, dim3((w.Np + 63) / 64, (rows + 15) / 16), dim3(256), 0, st, x, (const float*)w.w, w.Kp, w.Np, rows, out, rb, stride);
  LAUNCHCHK();
  *res = Slices{out, 1, (size_t)rows * w.Np, w.Np};
  return IXT_OK;
}
// gate | up product with the gated unit (IXT_GLU_*) behind it -> act(T) of the down product
template <typename T> static int hglu(ixt_ctx* c, const T* x, const HMat& w, size_t stride, int rows, int group_rows, const int32_t* rb, int kind, float limit, T* out, hipStream_t st);
template <> int hglu<bf16_t>(ixt_ctx* c, const bf16_t* x, const HMat& w, size_t stride, int rows, int group_rows, const int32_t* rb, int kind, float limit, bf16_t* out, hipStream_t st) {
  if (rb ? group_rows % 128 == 0 : rows >= c->ring_min_rows) {
    GemmEpi e{};
    e.act = out; e.glu = kind; e.glu_limit = limit; e.rb_exp = rb; e.wstride = stride / 8;
    return launch_ring(c, GEPI_SWIGLU, x, (const bf16_t*)w.w, w.Kp, w.Np, rows, e, false, st);
  }
  if (!rb && rows <= c->small_rows && sdot_plan(c, GEPI_SWIGLU, false, w.Kp, w.Np, rows).ok) {
    GemmEpi e{};
    e.act = out; e.glu = kind; e.glu_limit = limit;
    return launch_sdot(c, GEPI_SWIGLU, false, x, nullptr, (const bf16_t*)w.w, w.Kp, w.Np, rows, e, st);
  }
  const int rowblocks = (rows + 15) / 16, nrb = rb ? 1 : (rowblocks >= 3 ? 4 : rowblocks), zblocks = (rowblocks + nrb - 1) / nrb, ntile = w.Np / 16;
  dim3 grid((((ntile + 3) / 4 + 7) / 8) * 8 * zblocks, 1, 1);
  const u32x4 *xp = reinterpret_cast<const u32x4*>(x), *wp = reinterpret_cast<const u32x4*>(w.w);
  float* o = reinterpret_cast<float*>(out);
#define HGLU(B_, NT_) hipLaunchKernelGGL((k_dotb<B_, false, NT_, 1>), grid, dim3(256), (size_t)(B_) * 16 * 1024, st, xp, wp, w.Kp, w.Np, rows, o, ntile, zblocks, rb, stride / 8, kind, limit)
  if (nrb == 4) { if (zblocks == 1) HGLU(4, true); else HGLU(4, false); }
  else if (nrb == 2) HGLU(2, true);
  else HGLU(1, true);
#undef HGLU
  LAUNCHCHK();
  return IXT_OK;
}
template <> int hglu<float>(ixt_ctx* c, const float* x, const HMat& w, size_t stride, int rows, int, const int32_t* rb, int kind, float limit, float* out, hipStream_t st) {
  Slices t;
  TRY(hdot_grouped<float>(c, x, w, stride, rows, 16, rb, c->part, c->part_floats, st, &t));
  hipLaunchKernelGGL((k_glu_slices<float>), dim3(rows, (w.Np / 2 + 255) / 256), dim3(256), 0, st, t, w.Np / 2, kind, limit, out, rb);
  LAUNCHCHK();
  return IXT_OK;
}

template <int RT, int RS>
static int latent_launch(bool tall, int H, int splits, LatentAttnArgs a, hipStream_t st) {
  constexpr size_t tile = LatentTile<RT, RS>::BYTES;
  static bool attr_done = false;
  if (!attr_done) {
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_latent_attn<RT, RS>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)(2 * tile)));
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_latent_decode<RT, RS>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)tile));
    attr_done = true;
  }
  if (tall) {
    a.HB = std::min(H, 64); a.NQ = std::max(1, 64 / a.HB);
    hipLaunchKernelGGL((k_latent_attn<RT, RS>), dim3((a.R + a.NQ - 1) / a.NQ, (H + a.HB - 1) / a.HB), dim3(256), 2 * tile, st, a);
  } else {
    const int hg = (H + 15) / 16;
    a.HB = (H + hg - 1) / hg; a.NQ = 1;
    hipLaunchKernelGGL((k_latent_decode<RT, RS>), dim3(a.R, (H + a.HB - 1) / a.HB, splits), dim3(256), tile, st, a);
  }
  LAUNCHCHK();
  return IXT_OK;
}
// queries (slices in latent space + rotated parts) over the paged latents -> the value latents, act(T) row h Rp + r
template <typename T>
static int latent_attention(ixt_ctx* c, const HLayer& L, const Slices& qa, int R, int Rp, bool decode, int len_hint, hipStream_t st) {
  HybridModel* m = c->hy;
  const LatentGeom& g = L.lg;
  const int Kp = up_to(g.rankp, IXT_KALIGN);
  if constexpr (sizeof(T) == 2) {
    if (latent_mfma_fits(*m, g)) {
      const bool tall = !decode && R > 32;
      const int hg = (g.H + 15) / 16, span = g.window > 0 ? std::min(g.window, len_hint) : len_hint;
      int splits = 1;
      if (!tall) splits = std::min(std::min(16, std::max(1, 512 / (R * hg))), std::max(1, (span + 63) / 64));     // two blocks per CU, at least a tile each
      LatentAttnArgs a{qa, (const bf16_t*)m->qr, g, c->row_slot, c->row_pos, c->row_active, c->ps.page_map, (const bf16_t*)L.pages, R, Rp, 1, 1, __builtin_ctz(c->P), (bf16_t*)m->olat, Kp, m->po, m->pml};
      int rc = IXT_ERR_UNSUPPORTED;
      if (g.rotp == 32) {
        if (g.rankp == 64) rc = latent_launch<4, 1>(tall, g.H, splits, a, st);
        else if (g.rankp == 128) rc = latent_launch<8, 1>(tall, g.H, splits, a, st);
        else if (g.rankp == 256) rc = latent_launch<16, 1>(tall, g.H, splits, a, st);
        else rc = latent_launch<32, 1>(tall, g.H, splits, a, st);
      } else {
        if (g.rankp == 64) rc = latent_launch<4, 2>(tall, g.H, splits, a, st);
        else if (g.rankp == 128) rc = latent_launch<8, 2>(tall, g.H, splits, a, st);
        else if (g.rankp == 256) rc = latent_launch<16, 2>(tall, g.H, splits, a, st);
        else rc = latent_launch<32, 2>(tall, g.H, splits, a, st);
      }
      TRY(rc);
      if (splits > 1) {
        hipLaunchKernelGGL(k_latent_combine, dim3(R, g.H), dim3(128), 0, st, m->po, m->pml, splits, g.rankp, g.H, Rp, c->row_active, (bf16_t*)m->olat, Kp);
        LAUNCHCHK();
      }
      return IXT_OK;
    }
  }
  hipLaunchKernelGGL((k_latent_attn_any<T>), dim3(R, g.H), dim3(256), sizeof(float) * (g.rankp + g.rotp + 256), st, qa, (const T*)m->qr, g, c->row_slot, c->row_pos, c->row_active,
                     c->ps.page_map, (const T*)L.pages, Rp, (T*)m->olat, Kp);
  LAUNCHCHK();
  return IXT_OK;
}

// The mixers leave the operand of the output projection in m->act.
template <typename T>
static int hybrid_mixer_latent(ixt_ctx* c, const HLayer& L, const HLayer& W, int R, int Rp, bool decode, int len_hint, hipStream_t st) {
  HybridModel* m = c->hy;
  const LatentGeom& g = L.lg;
  Slices t;
  TRY(hdot<T>(c, (const T*)m->xb, W.in, R, c->part, c->part_floats, st, &t));
  hipLaunchKernelGGL((k_latent_prep<T>), dim3(R, 1 + (g.H + 3) / 4), dim3(256), 0, st, t, L.d_off, g, W.cnorm, m->eps, L.rope_cos, L.rope_sin, c->row_slot, c->row_pos, c->row_active,
                     c->ps.page_map, (T*)L.pages, (T*)m->qx, W.uk.Kp, Rp, (T*)m->qr);
  LAUNCHCHK();
  TRY(hdot_grouped<T>(c, (const T*)m->qx, W.uk, W.uk_stride, g.H * Rp, Rp, m->head_rb, c->part, c->part_floats, st, &t));
  TRY(latent_attention<T>(c, L, t, R, Rp, decode, len_hint, st));
  TRY(hdot_grouped<T>(c, (const T*)m->olat, W.uv, W.uv_stride, g.H * Rp, Rp, m->head_rb, c->part, c->part_floats, st, &t));
  hipLaunchKernelGGL((k_heads_x<T>), dim3(R, (W.o.Kp + 255) / 256), dim3(256), 0, st, t, g.H, L.c.vdim, Rp, (T*)m->act, W.o.Kp);
  LAUNCHCHK();
  return IXT_OK;
}

template <int DK, int DV>
static int heads_prompt_launch(HeadsAttnArgs a, hipStream_t st) {
  constexpr int lds = 2 * 64 * (DK + DV) * 2;
  static bool attr_done = false;
  if (!attr_done) {
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_heads_prompt<DK, DV>), hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    attr_done = true;
  }
  const int GQ = a.g.H / a.g.G;
  a.HB = std::min(GQ, 64); a.NQ = 64 / a.HB; a.hchunks = (GQ + a.HB - 1) / a.HB;
  hipLaunchKernelGGL((k_heads_prompt<DK, DV>), dim3(a.g.G * a.hchunks, (a.R + a.NQ - 1) / a.NQ), dim3(256), lds, st, a);
  LAUNCHCHK();
  return IXT_OK;
}
template <int DK, int DV>
static int heads_launch(bool tall, bool fused, int splits, HeadsAttnArgs a, hipStream_t st) {
  if (tall) return heads_prompt_launch<DK, DV>(a, st);
  constexpr int lds = 64 * (DK + DV) * 2;
  static bool attr_done = false;
  if (!attr_done) {
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_heads_decode<DK, DV, true>), hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    HIPCHK(hipFuncSetAttribute(reinterpret_cast<const void*>(&k_heads_decode<DK, DV, false>), hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    attr_done = true;
  }
  const dim3 grid(a.R, a.g.G * a.hchunks, splits);
  if (fused) hipLaunchKernelGGL((k_heads_decode<DK, DV, true>), grid, dim3(256), lds, st, a);
  else hipLaunchKernelGGL((k_heads_decode<DK, DV, false>), grid, dim3(256), lds, st, a);
  LAUNCHCHK();
  return IXT_OK;
}
template <typename T>
static int heads_prep(ixt_ctx* c, const HLayer& L, const HLayer& W, const Slices& t, const HeadsRope& rope, const RowsArgs& rows, int R, hipStream_t st) {
  HybridModel* m = c->hy;
  const HeadsGeom& g = L.hg;
  const int n = g.H + 2 * g.G, widest = std::max(g.dkp, g.vs);
#define HPREP(LP_) hipLaunchKernelGGL((k_heads_prep<T, LP_>), dim3(R, (n * LP_ + 255) / 256), dim3(256), 0, st, t, g, W.qn, W.kn, m->eps, rope, rows, (T*)L.pages, (T*)L.vpages, (T*)m->qx)
  if (widest <= 64) HPREP(16); else if (widest <= 128) HPREP(32); else HPREP(64);
#undef HPREP
  LAUNCHCHK();
  return IXT_OK;
}
template <typename T>
static int hybrid_mixer_heads(ixt_ctx* c, const HLayer& L, const HLayer& W, int R, bool decode, int len_hint, hipStream_t st) {
  HybridModel* m = c->hy;
  const HeadsGeom& g = L.hg;
  const RowsArgs rows{c->row_slot, c->row_pos, c->row_active, c->ps.page_map};
  const HeadsRope rope{L.rope_cos, L.rope_sin};
  Slices t;
  int dkp = 0, dvp = 0;
  TRY(hdot<T>(c, (const T*)m->xb, W.in, R, c->part, c->part_floats, st, &t));
  if constexpr (sizeof(T) == 2) {
    if (heads_mfma_sizes(g.d, g.dv, m->f32, &dkp, &dvp)) {
      const bool tall = !decode && R > 32;
      const int GQ = g.H / g.G, hchunks = (GQ + 15) / 16, blocks = R * g.G * hchunks, span = g.window > 0 ? std::min(g.window, len_hint) : len_hint;
      int splits = 1;
      if (!tall) splits = std::min(std::min(16, std::max(1, IXT_HEADS_SPLIT_BLOCKS / blocks)), std::max(1, (span + 63) / 64));     // at least a tile each
      if (!decode) TRY((heads_prep<T>(c, L, W, t, rope, rows, R, st)));
      HeadsAttnArgs a{(const bf16_t*)m->qx, g, W.sink, rows, (bf16_t*)L.pages, (bf16_t*)L.vpages, R, 1, (GQ + hchunks - 1) / hchunks, hchunks, __builtin_ctz(c->P),
                      (bf16_t*)m->act, W.o.Kp, m->po, m->pml, t, W.qn, W.kn, m->eps, rope};
      int rc = IXT_ERR_UNSUPPORTED;
#define X(DK_, DV_) if (dkp == DK_ && dvp == DV_) rc = heads_launch<DK_, DV_>(tall, decode, splits, a, st);
      IXT_HEADS_SIZES(X)
#undef X
      TRY(rc);
      if (splits > 1) {
        hipLaunchKernelGGL(k_heads_combine, dim3(R, g.H), dim3(64), 0, st, m->po, m->pml, splits, g.dvp, g.H, g.vs, c->row_active, (bf16_t*)m->act, W.o.Kp);
        LAUNCHCHK();
      }
      return IXT_OK;
    }
  }
  TRY((heads_prep<T>(c, L, W, t, rope, rows, R, st)));
  hipLaunchKernelGGL((k_heads_any<T>), dim3(R, g.H), dim3(256), sizeof(float) * (g.dkp + 256), st, (const T*)m->qx, g, W.sink, rows, (const T*)L.pages, (const T*)L.vpages, (T*)m->act, W.o.Kp);
  LAUNCHCHK();
  return IXT_OK;
}

template <typename T>
static int hybrid_mixer_delta(ixt_ctx* c, const HLayer& L, const HLayer& W, int R, int nseg_max, bool single, hipStream_t st) {
  HybridModel* m = c->hy;
  const DeltaGeom& g = L.dg;
  Slices t, t2;
  TRY(hdot<T>(c, (const T*)m->xb, W.in, R, c->part, c->part_floats, st, &t));
  hipLaunchKernelGGL((k_lowrank_x<T>), dim3(R), dim3(128), 0, st, t, g, (T*)m->act, W.low.Kp);
  LAUNCHCHK();
  TRY(hdot<T>(c, (const T*)m->act, W.low, R, m->part2, m->part2_floats, st, &t2));
  if (single) {            // every row is a segment of one token
    DeltaStepArgs da{t, t2, g, W.cq, W.ck, W.cv, W.a_log, W.dt_bias, W.onorm, m->eps, c->row_active, c->row_slot, c->row_pos, m->parity, L.tails, L.state};
    const dim3 grid(R, g.H);
    const size_t lds = sizeof(float) * (3 * g.dp + 2 * g.dv);
#define HSTEP(RP_) case RP_: hipLaunchKernelGGL((k_delta_step<T, RP_>), grid, dim3(256), lds, st, da, (T*)m->act, W.o.Kp); break
    switch (g.dp / 16) { HSTEP(1); HSTEP(2); HSTEP(4); HSTEP(8); HSTEP(16); HSTEP(32); default: return set_err(IXT_ERR_UNSUPPORTED, "delta rule: %d key dims", g.d); }
#undef HSTEP
    LAUNCHCHK();
    return IXT_OK;
  }
  DeltaPrepArgs pa{t, t2, g, W.cq, W.ck, W.cv, W.a_log, W.dt_bias, m->row_seg, m->row_j, m->seg, L.tails, m->dq, m->dk, m->dkq, m->dv, m->dec, m->beta};
  hipLaunchKernelGGL(k_delta_prep, dim3(R, (g.KH + g.H + 3) / 4), dim3(256), 0, st, pa);
  LAUNCHCHK();
  DeltaScanArgs sa{g, m->seg, m->nseg, m->dq, m->dk, m->dkq, m->dv, m->dec, m->beta, L.state, m->dout};
  const dim3 grid(nseg_max, g.H, (g.dv + 15) / 16);
#define HSCAN(RP_) case RP_: hipLaunchKernelGGL((k_delta_scan<RP_>), grid, dim3(256), sizeof(float) * 6 * scan_tokens<RP_>() * 16 * RP_, st, sa); break
  switch (g.dp / 16) { HSCAN(1); HSCAN(2); HSCAN(4); HSCAN(8); HSCAN(16); HSCAN(32); default: return set_err(IXT_ERR_UNSUPPORTED, "delta rule: %d key dims", g.d); }
#undef HSCAN
  LAUNCHCHK();
  hipLaunchKernelGGL((k_delta_out<T>), dim3(R, (g.H + 3) / 4), dim3(256), 0, st, m->dout, t2, g, W.onorm, m->eps, m->row_seg, (T*)m->act, W.o.Kp);
  LAUNCHCHK();
  return IXT_OK;
}

// routed mixture (and its shared unit: slices `shared`): expert outputs stay in copy order (slices `out`, row m->mpos[r top + j], weight m->mw[r top + j]); the norm kernel adds them up
template <typename T>
static int hybrid_moe(ixt_ctx* c, const HLayer& L, const HLayer& W, int R, hipStream_t st, Slices* out, Slices* shared) {
  HybridModel* m = c->hy;
  const ixt_layer& l = L.c;
  const int pairs = R * l.top, n = l.experts;
  const RouteRule rule{l.experts, l.top, l.router, l.groups > 1 ? l.groups : 0, l.groups_keep, l.router_norm, l.router_scale, W.corr};
  if (l.shared_ff > 0) {
    TRY(hglu<T>(c, (const T*)m->xb, W.sgu, 0, R, 0, nullptr, l.glu, l.glu_limit, (T*)m->hact, st));
    TRY(hdot<T>(c, (const T*)m->hact, W.sdown, R, m->part2, m->part2_floats, st, shared));
  }
  const float* h = (m->norm_places & IXT_NORM_BEFORE) ? m->h32 : m->x;
  const size_t lds = sizeof(float) * (l.experts + 2 * rule.groups);
  if (R <= 256) hipLaunchKernelGGL((k_route<1>), dim3(R), dim3(256), lds, st, h, W.router, m->E, m->Ep, rule, R, m->midx, m->mw);
  else hipLaunchKernelGGL((k_route<4>), dim3((R + 3) / 4), dim3(256), 4 * lds, st, h, W.router, m->E, m->Ep, rule, R, m->midx, m->mw);
  LAUNCHCHK();
  const int align = (m->f32 || pairs <= 64) ? 16 : 128;
  const int rows_g = up_to(pairs, align) + align * std::min(n, pairs);     // every expert with a copy may waste up to align - 1 rows
  if (rows_g > m->moe_cap) return set_err(IXT_ERR_INVALID, "moe: %d copies exceed the routed workspaces", pairs);
  hipLaunchKernelGGL(k_moe_plan_any, dim3(1), dim3(1024), 0, st, m->midx, pairs, n, align, rows_g / 16, m->mpos, m->mrb);
  if constexpr (sizeof(T) == 2) hipLaunchKernelGGL(k_moe_gather, dim3(pairs, (m->Ep + 2047) / 2048), dim3(256), 0, st, (const bf16_t*)m->xb, m->mpos, l.top, m->Ep, (bf16_t*)m->xg);
  else hipLaunchKernelGGL(k_gather32, dim3(pairs, (m->Ep + 255) / 256), dim3(256), 0, st, (const float*)m->xb, m->mpos, l.top, m->Ep, (float*)m->xg);
  LAUNCHCHK();
  TRY(hglu<T>(c, (const T*)m->xg, W.gu, W.gu_stride, rows_g, align, m->mrb, l.glu, l.glu_limit, (T*)m->mhact, st));
  return hdot_grouped<T>(c, (const T*)m->mhact, W.down, W.down_stride, rows_g, align, m->mrb, c->part, c->part_floats, st, out);
}

// logits of rows lrows[i] (or lrow0 + i) of the residual stream, NLmax at a time
template <typename T>
static int hybrid_logits(ixt_ctx* c, int R, int lrow0, int nl, const int32_t* lrows, int32_t* argmax_out, float* logits_out, hipStream_t st) {
  HybridModel* m = c->hy;
  const int nblk = (m->V + 1023) / 1024;
  for (int i0 = 0; i0 < nl; i0 += c->NLmax) {
    const int n = std::min(c->NLmax, nl - i0);
#define HFINAL(KIND_) hipLaunchKernelGGL((k_final_norm<T, KIND_>), dim3(n), dim3(256), 0, st, m->x, lrows ? lrows + i0 : nullptr, lrow0 + i0, R, m->fnorm, m->eps, m->E, m->Ep, (T*)m->xn)
    if (m->norm_kind == IXT_NORM_TANH) HFINAL(IXT_NORM_TANH); else HFINAL(IXT_NORM_RMS);
#undef HFINAL
    LAUNCHCHK();
    Slices t;
    TRY(hdot<T>(c, (const T*)m->xn, m->head, n, c->part, c->part_floats, st, &t));
    hipLaunchKernelGGL(k_head_post, dim3(nblk, n), dim3(256), 0, st, t, m->V, c->sample_cols, logits_out ? logits_out + (size_t)i0 * m->V : nullptr, c->amax_val, c->amax_idx);
    if (argmax_out) hipLaunchKernelGGL(k_argmax_final, dim3(n), dim3(256), 0, st, c->amax_val, c->amax_idx, nblk, argmax_out + i0);
    LAUNCHCHK();
  }
  return IXT_OK;
}

// x <- x + post(t), the next operand pre(x) (k_sub_norm); routed: its f32 copy too
template <typename T>
static int hybrid_norm(ixt_ctx* c, const Slices& t, const Slices& add, const int32_t* pos, const float* wts, int top, const NormW& post, const NormW& pre, bool routed, int R, hipStream_t st) {
  HybridModel* m = c->hy;
  float* h32 = routed && pre.w != nullptr ? m->h32 : nullptr;
#define HNORM(NI_, KIND_) hipLaunchKernelGGL((k_sub_norm<T, NI_, KIND_>), dim3(R), dim3(256), 0, st, t, add, pos, wts, top, post, pre, m->eps, m->E, m->Ep, m->x, (T*)m->xb, h32)
#define HNORM_K(NI_) do { if (m->norm_kind == IXT_NORM_TANH) HNORM(NI_, IXT_NORM_TANH); else HNORM(NI_, IXT_NORM_RMS); } while (0)
  if (m->Ep <= 2048) HNORM_K(1); else if (m->Ep <= 4096) HNORM_K(2); else if (m->Ep <= 8192) HNORM_K(4); else HNORM_K(6);
#undef HNORM_K
#undef HNORM
  LAUNCHCHK();
  return IXT_OK;
}

// a sublayer's last product and what follows it: x <- x + post(W v), the next operand pre(x).  Tanh norms ride in the product's epilogue where the whole
// sum is in one place.
template <typename T>
static int hybrid_dot_norm(ixt_ctx* c, const T* v, const HMat& w, const NormW& post, const NormW& pre, bool routed, int R, hipStream_t st) {
  HybridModel* m = c->hy;
  if constexpr (sizeof(T) == 2) {
    const bool small = R <= c->small_rows && sdot_plan(c, GEPI_TANHNORM, false, w.Kp, w.Np, R).ok;
    if (m->norm_kind == IXT_NORM_TANH && (small || R >= c->ring_min_rows)) {
      GemmEpi e{};
      e.act = (bf16_t*)m->xb;
      e.tn = TanhNormEpi{post.w, post.b, post.alpha, pre.w, pre.b, pre.alpha, m->x, routed && pre.w != nullptr ? m->h32 : nullptr, m->E, m->Ep};
      if (small) return launch_sdot(c, GEPI_TANHNORM, false, v, nullptr, (const bf16_t*)w.w, w.Kp, w.Np, R, e, st);
      return launch_ring(c, GEPI_TANHNORM, v, (const bf16_t*)w.w, w.Kp, w.Np, R, e, false, st);
    }
  }
  Slices t;
  TRY(hdot<T>(c, v, w, R, c->part, c->part_floats, st, &t));
  return hybrid_norm<T>(c, t, Slices{}, nullptr, nullptr, 0, post, pre, routed, R, st);
}

template <typename T>
static int forward_rows_hybrid_t(ixt_ctx* c, int R, const int32_t* tokens, int len_hint, int lrow0, int nl, const int32_t* lrows, int32_t* argmax_out, float* logits_out, bool decode,
                                 int nseg_max, hipStream_t st) {
  HybridModel* m = c->hy;
  const int Rp = (sizeof(T) == 2 && R >= c->ring_min_rows) ? up_to(R, 128) : up_to(R, 16);
  if (m->recurrent || m->maxH > 0)
    hipLaunchKernelGGL(k_segments, dim3(1), dim3(1024), 0, st, R, c->row_active, c->row_slot, c->row_pos, m->row_seg, m->row_j, m->seg, m->nseg, m->state_len, m->parity, m->claim, c->G,
                     m->recurrent ? 1 : 0, m->err, m->head_rb, m->maxH * (Rp / 16), Rp / 16);
  const NormW none{}, first = m->layers[m->layers[0].src].n1;
  hipLaunchKernelGGL((k_embed_scaled<T>), dim3(R), dim3(256), 0, st, (const T*)m->embed, tokens, m->emb_scale, m->E, m->Ep, m->V, m->norm_kind == IXT_NORM_TANH ? first : none, m->x, (T*)m->xb);
  LAUNCHCHK();
  if (m->norm_kind == IXT_NORM_RMS && first.w != nullptr) TRY((hybrid_norm<T>(c, Slices{}, Slices{}, nullptr, nullptr, 0, none, first, false, R, st)));
  for (size_t i = 0; i < m->layers.size(); ++i) {
    const HLayer& L = m->layers[i];
    const HLayer& W = m->layers[L.src];
    if (L.c.mixer == IXT_MIX_LATENT_ATTENTION) TRY((hybrid_mixer_latent<T>(c, L, W, R, Rp, decode, len_hint, st)));
    else if (L.c.mixer == IXT_MIX_ATTENTION) TRY((hybrid_mixer_heads<T>(c, L, W, R, decode, len_hint, st)));
    else TRY((hybrid_mixer_delta<T>(c, L, W, R, nseg_max, decode, st)));
    const NormW next = i + 1 < m->layers.size() ? m->layers[m->layers[i + 1].src].n1 : none;      // (the head's norm is taken of the wanted rows only)
    TRY((hybrid_dot_norm<T>(c, (const T*)m->act, W.o, W.n1b, L.c.ffn == IXT_FFN_NONE ? next : W.n2, L.c.ffn == IXT_FFN_MOE, R, st)));
    if (L.c.ffn == IXT_FFN_DENSE) {
      TRY(hglu<T>(c, (const T*)m->xb, W.gu, 0, R, 0, nullptr, L.c.glu, L.c.glu_limit, (T*)m->hact, st));
      TRY((hybrid_dot_norm<T>(c, (const T*)m->hact, W.down, W.n2b, next, false, R, st)));
    } else if (L.c.ffn == IXT_FFN_MOE) {
      Slices t, shared{};
      TRY(hybrid_moe<T>(c, L, W, R, st, &t, &shared));
      if (t.n > 2 && R <= 64) {
        hipLaunchKernelGGL(k_moe_sum, dim3((t.ncols + 255) / 256, R), dim3(64), 0, st, t, m->mpos, m->mw, L.c.top, m->msum);
        LAUNCHCHK();
        TRY((hybrid_norm<T>(c, Slices{m->msum, 1, 0, t.ncols}, shared, nullptr, nullptr, 0, W.n2b, next, false, R, st)));
      } else {
        TRY((hybrid_norm<T>(c, t, shared, m->mpos, m->mw, L.c.top, W.n2b, next, false, R, st)));
      }
    }
    if (m->tap && !c->capturing) {
      if ((i + 1) * (size_t)R * m->E > m->tap_floats) return set_err(IXT_ERR_INVALID, "residual tap: buffer too small");
      HIPCHK(hipMemcpyAsync(m->tap + i * (size_t)R * m->E, m->x, sizeof(float) * (size_t)R * m->E, hipMemcpyDeviceToDevice, st));
    }
  }
  c->h_final_rows = R;
  if (nl > 0) TRY((hybrid_logits<T>(c, R, lrow0, nl, lrows, argmax_out, logits_out, st)));
  return IXT_OK;
}
int forward_rows_hybrid(ixt_ctx* c, int R, const int32_t* tokens, int len_hint, int lrow0, int nl, const int32_t* lrows, int32_t* argmax_out, float* logits_out, bool decode,
                               hipStream_t st) {
  const int nseg_max = decode ? R : std::min(R, c->one_segment ? 1 : c->G);     // a page group has at most one run of rows in a call
  if (c->hy->f32) return forward_rows_hybrid_t<float>(c, R, tokens, len_hint, lrow0, nl, lrows, argmax_out, logits_out, decode, nseg_max, st);
  return forward_rows_hybrid_t<bf16_t>(c, R, tokens, len_hint, lrow0, nl, lrows, argmax_out, logits_out, decode, nseg_max, st);
}

HybridModel* hybrid_new() { return new HybridModel(); }
void hybrid_free(ixt_ctx* c) { delete c->hy; c->hy = nullptr; }
bool hybrid_complete(const ixt_ctx* c) { return c->hy->missing == 0; }
int hybrid_prompt_logits(ixt_ctx* c, int row0, int n, hipStream_t st) {       // rows of the last pass's residual stream -> c->plogits
  if (c->hy->f32) return hybrid_logits<float>(c, c->h_final_rows, row0, n, nullptr, c->pargmax, c->plogits, st);
  return hybrid_logits<bf16_t>(c, c->h_final_rows, row0, n, nullptr, c->pargmax, c->plogits, st);
}
extern "C" int ixt_state_status(ixt_ctx* c, int32_t* out1, int reset, void* stream) {
  if (!c || !out1) return set_err(IXT_ERR_INVALID, "null argument");
  *out1 = 0;
  if (!c->hy) return IXT_OK;
  hipStream_t st = (hipStream_t)stream;
  HIPCHK(hipMemcpyAsync(out1, c->hy->err, sizeof(int32_t), hipMemcpyDeviceToHost, st));
  HIPCHK(hipStreamSynchronize(st));
  if (reset && *out1 != 0) HIPCHK(hipMemsetAsync(c->hy->err, 0, sizeof(int32_t), st));
  return IXT_OK;
}
extern "C" int ixt_set_residual_tap(ixt_ctx* c, float* dev, int64_t floats) {
  if (!c || !c->hy) return set_err(IXT_ERR_UNSUPPORTED, "the residual tap is built for hybrid decoders");
  c->hy->tap = dev; c->hy->tap_floats = dev ? (size_t)floats : 0;
  return IXT_OK;
}
