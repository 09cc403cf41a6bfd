// ixt_hybrid.hip -- host side of IXT_BLOCK_HYBRID: layer plans, weight loading, caches and states, and the forward pass over rows that every engine
// entry point (prefill chunk, packed rows, decode step) ends in.
#include "ixt_hybrid.h"

// what one latent row is padded to: the matrix-core kernel's sizes, beyond them multiples of 32 (k_latent_attn_any)
static int latent_rankp(int rank) { return rank <= 64 ? 64 : rank <= 128 ? 128 : rank <= 256 ? 256 : rank <= 512 ? 512 : up_to(rank, 32); }
static int latent_rotp(int rot) { return rot <= 32 ? 32 : rot <= 64 ? 64 : up_to(rot, 32); }
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
// of every `group` columns the `rot` from r0 on turn in pairs (ixt_layer.rope_pairs): the kernels want those side by side
static LoadMap rotated(LoadMap m, const ixt_layer& l, int group, int r0) {
  if (l.rope_pairs == IXT_ROPE_HALVES && l.rot_dim > 0) { m.rg = group; m.r0 = r0; m.rn = l.rot_dim; }
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
// [n][k] -> rows of kp elements (zeros behind k are there already)
static int h_load_rows(const HybridModel* m, const void* src, int dtype, void* dst, int64_t n, int64_t k, int64_t kp, hipStream_t st) {
  const unsigned blocks = (unsigned)((n * k + 255) / 256);
#define HROWS(S_, T_) hipLaunchKernelGGL((k_load_rows<S_, T_>), dim3(blocks), dim3(256), 0, st, (const S_*)src, (T_*)dst, n, k, kp)
  if (dtype == IXT_BF16) { if (m->f32) HROWS(bf16_t, float); else HROWS(bf16_t, bf16_t); }
  else if (dtype == IXT_F32) { if (m->f32) HROWS(float, float); else HROWS(float, bf16_t); }
  else return set_err(IXT_ERR_INVALID, "dtype %d", dtype);
#undef HROWS
  LAUNCHCHK();
  return IXT_OK;
}
static int h_load_mat(const HybridModel* m, const void* src, int dtype, void* dst, const LoadMap& lm, hipStream_t st) {
  return m->f32 ? h_load_nk(src, dtype, (float*)dst, lm, st) : h_load_nk(src, dtype, (bf16_t*)dst, lm, st);
}

static bool column_mixer(const ixt_layer& l) { return l.mixer == IXT_MIX_ATTENTION || l.mixer == IXT_MIX_RETENTION || l.mixer == IXT_MIX_LIGHTNING; }      // columns of one input projection, rows of one output projection
static int check_mixer(const ixt_layer& l, int i) {
  if (l.heads < 1 || l.dim < 1 || l.vdim < 1) return set_err(IXT_ERR_INVALID, "layer %d: heads / dim / vdim", i);
  if (l.rope_pairs != IXT_ROPE_NEIGHBOURS && l.rope_pairs != IXT_ROPE_HALVES) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: rope_pairs %d", i, l.rope_pairs);
  if (l.mixer == IXT_MIX_LATENT_ATTENTION) {
    if (l.kv_rank < 1 || l.kv_rank > 1024 || l.rot_dim < 0 || l.rot_dim % 2 || l.q_rank < 0)
      return set_err(IXT_ERR_UNSUPPORTED, "layer %d: kv_rank %d (1 .. 1024), rot_dim %d (even), q_rank %d", i, l.kv_rank, l.rot_dim, l.q_rank);
  } else if (l.mixer == IXT_MIX_GATED_DELTA) {
    if (l.kv_heads < 1 || l.heads % l.kv_heads || l.conv < 1 || l.decay_rank < 1 || l.gate_rank < 1) return set_err(IXT_ERR_INVALID, "layer %d: kv_heads / conv / ranks", i);
    if (l.dim > 512) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: delta rule key dims %d (at most 512)", i, l.dim);
  } else if (l.mixer == IXT_MIX_ATTENTION) {
    if (l.kv_heads < 1 || l.heads % l.kv_heads || l.rot_dim < 0 || l.rot_dim % 2 || l.rot_dim > l.dim) return set_err(IXT_ERR_INVALID, "layer %d: kv_heads / rot_dim", i);
    if (l.maps < 0 || l.maps > 2 || !(l.softcap >= 0.0f)) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: %d maps (1, 2), soft cap %g", i, l.maps, l.softcap);
    if (l.dim > 4096 || l.vdim > 1024) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: %d key dims (at most 4096), %d value dims (at most 1024)", i, l.dim, l.vdim);
    if (!(l.attn_scale > 0.0f)) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: score factor %g (positive)", i, l.attn_scale);
    if (l.rope_factor > 0.0f && !(l.rope_low > 0.0f && l.rope_high > l.rope_low && l.rope_original > 0.0f)) return set_err(IXT_ERR_INVALID, "layer %d: rotation scaling", i);
    if (l.key_values && (l.maps > 1 || l.dim != l.vdim)) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: keys as values with %d maps, %d key and %d value dims", i, l.maps, l.dim, l.vdim);
    if (l.chunk > 0 && l.window > 0) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: chunks of %d and a window of %d", i, l.chunk, l.window);
    if (l.qk_norm < 0 || l.qk_norm > 2 || l.out_gate < 0 || l.out_gate > 2) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: qk_norm %d, out_gate %d", i, l.qk_norm, l.out_gate);
  } else if (l.mixer == IXT_MIX_RETENTION || l.mixer == IXT_MIX_LIGHTNING) {
    if (!l.decay || l.rot_dim < 0 || l.rot_dim % 2 || l.rot_dim > l.dim) return set_err(IXT_ERR_INVALID, "layer %d: decays / rot_dim", i);
    if (l.dim > 1024 || l.vdim > 1024) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: %d key dims, %d value dims (at most 1024)", i, l.dim, l.vdim);
  } else if (l.mixer == IXT_MIX_SCAN) {
    if (l.inner < 1 || l.state < 1 || l.dt_rank < 1 || l.conv < 1) return set_err(IXT_ERR_INVALID, "layer %d: inner / state / dt_rank / conv", i);
    if (l.state > 256) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: %d states per channel (at most 256)", i, l.state);
  } else return set_err(IXT_ERR_UNSUPPORTED, "layer %d: mixer %d", i, l.mixer);
  if (l.mix_scale != 1.0f && !column_mixer(l)) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: a factor on mixer %d", i, l.mixer);
  return IXT_OK;
}

int hybrid_check(const ixt_config& c) {
  if (!c.layers || c.num_decoder_layers < 1) return set_err(IXT_ERR_INVALID, "hybrid decoder: no layers");
  if (c.emb_dim < 1 || c.emb_dim > 12288 || c.vocab_size < 1) return set_err(IXT_ERR_UNSUPPORTED, "hybrid decoder: emb_dim %d (1 .. 12288), vocab_size %d", c.emb_dim, c.vocab_size);
  if (c.fp8_weights) return set_err(IXT_ERR_UNSUPPORTED, "hybrid decoder: fp8 weights are not built");
  if (c.norm_kind < IXT_NORM_RMS || c.norm_kind > IXT_NORM_ONE || c.norm_places < IXT_NORM_BEFORE || c.norm_places > (IXT_NORM_BEFORE | IXT_NORM_AFTER))
    return set_err(IXT_ERR_UNSUPPORTED, "hybrid decoder: norm kind %d, places %d", c.norm_kind, c.norm_places);
  if (c.streams < 0 || c.streams > HC_MAX) return set_err(IXT_ERR_UNSUPPORTED, "hybrid decoder: %d streams (at most %d)", c.streams, HC_MAX);
  for (int i = 0; i < c.num_decoder_layers; ++i) {
    const ixt_layer& l = c.layers[i];
    if (l.weights_of >= c.num_decoder_layers || (l.weights_of >= 0 && c.layers[l.weights_of].weights_of >= 0) || l.weights_of == i)
      return set_err(IXT_ERR_INVALID, "layer %d: weights_of %d", i, l.weights_of);
    TRY(check_mixer(l, i));
    if (l.beside) {
      TRY(check_mixer(*l.beside, i));
      if (!column_mixer(l) || !column_mixer(*l.beside) || l.beside->beside || l.beside->mix_bias)
        return set_err(IXT_ERR_UNSUPPORTED, "layer %d: mixers %d and %d side by side (attention over heads, retention, lightning; output biases of the first one only)", i, l.mixer, l.beside->mixer);
    }
    if (l.loop_pass >= 0 && c.streams > 0) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: a pass with an input of its own among streams", i);
    if (l.shift && (c.streams > 0 || !(c.norm_places & IXT_NORM_BEFORE))) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: token shift among streams or without a norm in front", i);
    if (l.ffn != IXT_FFN_NONE && (l.glu < IXT_GLU_CLAMPED || l.glu > IXT_ACT_XIELU || (l.glu == IXT_ACT_XIELU && l.ffn != IXT_FFN_DENSE))) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: unit %d", i, l.glu);
    if (l.ffn == IXT_FFN_MOE) {
      if (l.experts < 1 || l.experts > 1024 || l.top < 1 || l.top > l.experts || l.ff < 1 || l.shared_ff < 0)
        return set_err(IXT_ERR_UNSUPPORTED, "layer %d: experts %d (1 .. 1024), top %d", i, l.experts, l.top);
      if (l.router < IXT_ROUTE_SOFTMAX || l.router > IXT_ROUTE_CHOSEN) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: router %d", i, l.router);
      if (l.groups > 1 && (l.experts % l.groups || l.groups_keep < 1 || l.groups_keep > l.groups || l.top > l.experts / l.groups * l.groups_keep))
        return set_err(IXT_ERR_INVALID, "layer %d: %d of %d groups of experts, top %d", i, l.groups_keep, l.groups, l.top);
    } else if (l.ffn == IXT_FFN_DENSE) {
      if (l.ff < 1) return set_err(IXT_ERR_INVALID, "layer %d: ff", i);
    } else if (l.ffn != IXT_FFN_NONE) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: ffn %d", i, l.ffn);
  }
  return IXT_OK;
}

// a norm's tensors: `name` (IXT_NORM_ONE: a scalar), name.b (tanh and layer norms), name.alpha (tanh norms: a scalar); zeros behind the E features
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
  if (m->norm_kind == IXT_NORM_ONE) return one(name, &w->w, 1, {});
  TRY(one(name, &w->w, E, {E}));
  if (m->norm_kind == IXT_NORM_TANH) TRY(one(name + ".alpha", &w->alpha, 1, {}));
  if (m->norm_kind != IXT_NORM_RMS) TRY(one(name + ".b", &w->b, E, {E}));
  return IXT_OK;
}

// parameters of layer i (its own tensors; a layer with weights_of has none)
static int hybrid_layer_params(ixt_ctx* c, int i) {
  HybridModel* m = c->hy;
  HLayer& L = m->layers[i];
  const ixt_layer& l = L.c;
  const int E = m->E;
  const std::string p = "l" + std::to_string(l.number < 0 ? i : l.number) + ".";
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
  auto hyper = [&](const std::string& q, float** dst, bool used) -> int {         // a sublayer's hyper-connection
    if (m->streams == 0) return IXT_OK;
    const int S = m->streams;
    float* d = nullptr;
    if (used) TRY(h_allocf(c, &d, 2 * HC_MAX + HC_MAX * HC_MAX));
    *dst = d;
    const std::vector<std::pair<std::string, LoadMap>> parts = {{"in", load_map(1, S, HC_MAX)}, {"out", load_map(1, S, HC_MAX)}, {"mix", load_map(S, S, HC_MAX)}};
    for (int j = 0; j < 3; ++j) {
      const LoadMap lm = parts[j].second;
      float* to = d + j * HC_MAX;
      const std::vector<int64_t> shape = j < 2 ? std::vector<int64_t>{S} : std::vector<int64_t>{S, S};
      if (used) add(q + parts[j].first, shape, [=](const void* s, int dt, hipStream_t st) { return h_load_nk(s, dt, to, lm, st); });
      else m->tensors[p + q + parts[j].first] = HTensor{shape, nullptr, true};
    }
    return IXT_OK;
  };
  // the tensors of a mixer that owns columns c0 .. of `in` and rows oc .. of `o`
  auto columns = [&](HLayer& X, const std::string& q) -> int {
    const ixt_layer& x = X.c;
    const HMat &in = L.in, &o = L.o;
    float* ib = L.ibias;
    auto bias = [&](const std::string& name, LoadMap lm) {
      lm.k = lm.ld = lm.Kp = 1;
      add(q + name, {lm.n}, [=](const void* s, int dt, hipStream_t st) { return h_load_nk(s, dt, ib, lm, st); });
    };
    if (x.mixer == IXT_MIX_ATTENTION) {
      const HeadsGeom& g = X.hg;
      LoadMap lq = load_map(g.H * g.maps * g.d, E, in.Kp, X.c0), lk = load_map(g.G * g.maps * g.d, E, in.Kp, X.c0 + g.ok), lv = load_map(g.G * g.dv, E, in.Kp, X.c0 + g.ov);
      lq.ng = lk.ng = g.d; lq.ngp = lk.ngp = g.hs; lv.ng = g.dv; lv.ngp = g.vs;
      lq = rotated(lq, x, g.d, 0); lk = rotated(lk, x, g.d, 0);
      mat_as(q + "q", in, lq);
      mat_as(q + "k", in, lk);
      if (!x.key_values) mat_as(q + "v", in, lv);
      if (x.mix_bias) {
        bias("q.b", lq); bias("k.b", lk);
        if (!x.key_values) bias("v.b", lv);
        TRY(h_allocf(c, &X.obias, (size_t)m->Ep));
        float* ob = X.obias;
        add(q + "o.b", {E}, [=](const void* s, int dt, hipStream_t st) { return h_load_vec(s, dt, ob, (int64_t)E, st); });
      }
      if (g.og >= 0) {
        LoadMap gm = load_map(g.head_gate ? g.H : g.H * g.dv, E, in.Kp, X.c0 + g.og);
        if (!g.head_gate) { gm.ng = g.dv; gm.ngp = g.vs; }
        mat_as(q + "g", in, gm);
      }
      if (g.maps == 2) {                                          // every one of the four vectors works lambda out anew: the last to come leaves the right one
        const int n = up_to(g.d, 4);
        TRY(h_allocf(c, &X.maps, (size_t)4 * n)); TRY(h_allocf(c, &X.lambda, 4));
        const char* names[4] = {"lq1", "lk1", "lq2", "lk2"};
        float *base = X.maps, *lam = X.lambda;
        const int d = g.d;
        const float diff = x.map_diff;
        for (int j = 0; j < 4; ++j) {
          float* to = base + (size_t)j * n;
          add(q + names[j], {d}, [=](const void* s, int dt, hipStream_t st) -> int {
            TRY(h_load_vec(s, dt, to, (int64_t)d, st));
            hipLaunchKernelGGL(k_maps_lambda, dim3(1), dim3(64), 0, st, base, base + n, base + 2 * n, base + 3 * n, d, diff, lam);
            LAUNCHCHK();
            return IXT_OK;
          });
        }
      }
      if (x.qk_norm == 2) {                                       // (one vector of ones serves both)
        TRY(h_allocf(c, &X.qn, (size_t)up_to(g.d, 4)));
        const std::vector<float> ones(g.d, 1.0f);
        HIPCHK(hipMemcpy(X.qn, ones.data(), ones.size() * 4, hipMemcpyHostToDevice));
        X.kn = X.qn;
      } else if (x.qk_norm) {
        for (int j = 0; j < 2; ++j) {
          float** dst = j == 0 ? &X.qn : &X.kn;
          TRY(h_allocf(c, dst, (size_t)up_to(g.d, 4)));
          float* d = *dst;
          const LoadMap lm = rotated(load_map(g.d, 1, 1), x, g.d, 0);
          add(q + (j == 0 ? "q.norm" : "k.norm"), {g.d}, [=](const void* s, int dt, hipStream_t st) { return h_load_nk(s, dt, d, lm, st); });
        }
      }
      if (x.sink) TRY(vec(q + "sink", &X.sink, g.H, {g.H}));
      LoadMap lo = load_map(E, g.H * g.dv, o.Kp, 0, g.oc);
      lo.kg = g.dv; lo.kgp = g.vs;
      if (x.key_values && lk.rn > 0) { lo.krg = g.d; lo.krn = lk.rn; }
      mat_as(q + "o", o, lo);
      return IXT_OK;
    }
    const RetGeom& g = X.rg;
    for (const char* t : {"q", "k", "v", "g"}) {
      const bool qk = *t == 'q' || *t == 'k';
      LoadMap lm = load_map(g.H * (qk ? g.d : g.dv), E, in.Kp, X.c0 + (*t == 'q' ? 0 : *t == 'k' ? g.ok : *t == 'v' ? g.ov : g.og));
      lm.ng = qk ? g.d : g.dv; lm.ngp = qk ? g.hs : g.vs;
      mat_as(q + t, in, qk ? rotated(lm, x, g.d, 0) : lm);
    }
    if (g.join_norm) {
      TRY(h_allocf(c, &X.onorm, (size_t)g.H * g.vs));
      float* d = X.onorm;
      LoadMap lm = load_map(g.H * g.dv, 1, 1);
      lm.ng = g.dv; lm.ngp = g.vs;
      add(q + "norm", {g.H * g.dv}, [=](const void* s, int dt, hipStream_t st) { return h_load_nk(s, dt, d, lm, st); });
    }
    LoadMap lo = load_map(E, g.H * g.dv, o.Kp, 0, g.oc);
    lo.kg = g.dv; lo.kgp = g.vs;
    mat_as(q + "o", o, lo);
    return IXT_OK;
  };
  TRY(hyper("hc1.", &L.hc1, true));
  TRY(hyper("hc2.", &L.hc2, l.ffn != IXT_FFN_NONE));
  const bool both = m->norm_places == (IXT_NORM_BEFORE | IXT_NORM_AFTER);
  TRY(norm("norm1", m->norm_places & IXT_NORM_BEFORE ? &L.n1 : &L.n1b));
  if (both) TRY(norm("norm1b", &L.n1b));
  if (l.shift) {
    TRY(h_allocf(c, &L.mu, (size_t)m->Ep));
    float* d = L.mu;
    add("shift", {E}, [=](const void* s, int dt, hipStream_t st) { return h_load_vec(s, dt, d, (int64_t)E, st); });
  }
  if (l.mixer == IXT_MIX_LATENT_ATTENTION) {
    const LatentGeom& g = L.lg;
    const int NQ = g.H * (g.dn + g.dr);
    TRY(h_mat(c, &L.in, E, l.out_gate ? L.g_off + g.H * l.vdim : L.d_off + g.rank + g.dr));
    if (l.q_rank > 0) {
      mat("mix.dq", L.in, l.q_rank, E, 0);
      TRY(vec("mix.dq.norm", &L.qnorm, l.q_rank, {l.q_rank}));
      TRY(h_mat(c, &L.uq, l.q_rank, NQ));
      mat_as("mix.uq", L.uq, rotated(load_map(NQ, l.q_rank, L.uq.Kp), l, g.dn + g.dr, g.dn));
    } else mat_as("mix.q", L.in, rotated(load_map(NQ, E, L.in.Kp), l, g.dn + g.dr, g.dn));
    mat_as("mix.dkv", L.in, rotated(load_map(g.rank + g.dr, E, L.in.Kp, L.d_off), l, g.rank + g.dr, g.rank));
    if (l.out_gate) mat("mix.g", L.in, g.H * l.vdim, E, L.g_off);
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
  } else if (column_mixer(l)) {
    TRY(h_mat(c, &L.in, E, L.in_cols));
    TRY(h_mat(c, &L.o, L.o_rows, E));
    if (l.mix_bias) TRY(h_allocf(c, &L.ibias, (size_t)L.in.Np));
    TRY(columns(L, L.side ? "mix.left." : "mix."));
    if (L.side) TRY(columns(*L.side, "mix.right."));
  } else if (l.mixer == IXT_MIX_SCAN) {
    const ScanGeom& g = L.sg;
    const int64_t C = g.C, N = g.N;
    TRY(h_mat(c, &L.in, E, g.oz + g.C));
    {
      HMat& M = L.in;
      char* d = (char*)M.w;
      const LoadMap x = load_map(g.C, E, M.Kp), z = load_map(g.C, E, M.Kp, g.oz);
      add("mix.in", {2 * C, E}, [=](const void* s, int dt, hipStream_t st) {
        TRY(h_load_mat(m, s, dt, d, x, st));
        return h_load_mat(m, (const char*)s + (size_t)C * E * (dt == IXT_F32 ? 4 : 2), dt, d, z, st);
      });
    }
    TRY(h_allocf(c, &L.cw, (size_t)g.taps * g.Cp));
    {
      float* d = L.cw;
      LoadMap lm = load_map(g.taps, g.C, g.Cp);                   // tap by tap
      lm.trans = 1; lm.ld = g.taps;
      add("mix.conv", {C, g.taps}, [=](const void* s, int dt, hipStream_t st) { return h_load_nk(s, dt, d, lm, st); });
    }
    TRY(vec("mix.conv.b", &L.cb, C, {C}));
    TRY(h_mat(c, &L.low, g.C, g.oc + g.N));
    {
      char* d = (char*)L.low.w;
      const LoadMap t = load_map(g.rank, g.C, L.low.Kp), b = load_map(g.N, g.C, L.low.Kp, g.ob), y = load_map(g.N, g.C, L.low.Kp, g.oc);
      const int rank = g.rank;
      add("mix.x", {rank + 2 * N, C}, [=](const void* s, int dt, hipStream_t st) {
        const size_t row = (size_t)C * (dt == IXT_F32 ? 4 : 2);
        TRY(h_load_mat(m, s, dt, d, t, st));
        TRY(h_load_mat(m, (const char*)s + rank * row, dt, d, b, st));
        return h_load_mat(m, (const char*)s + (rank + N) * row, dt, d, y, st);
      });
    }
    TRY(h_mat(c, &L.dt, g.rank, g.C));
    L.rankp = up_to(g.rank, 8);
    TRY(h_alloc(c, &L.dtw, (size_t)g.C * L.rankp * m->esz));
    {
      void *d = L.dt.w, *rows = L.dtw;
      const LoadMap lm = load_map(g.C, g.rank, L.dt.Kp);
      const int64_t wide = L.rankp, rank = g.rank;
      add("mix.dt", {C, g.rank}, [=](const void* s, int dt, hipStream_t st) -> int {
        TRY(h_load_mat(m, s, dt, d, lm, st));
        return h_load_rows(m, s, dt, rows, C, rank, wide, st);
      });
    }
    TRY(h_allocf(c, &L.dtb, (size_t)L.dt.Np)); TRY(h_allocf(c, &L.a2, (size_t)g.C * g.Np)); TRY(h_allocf(c, &L.D, (size_t)g.Cp));
    {
      float *b = L.dtb, *a2 = L.a2, *D = L.D;
      const int Np = g.Np;
      add("mix.dt.b", {C}, [=](const void* s, int dt, hipStream_t st) { return h_load_vec(s, dt, b, C, st); });
      add("mix.D", {C}, [=](const void* s, int dt, hipStream_t st) { return h_load_vec(s, dt, D, C, st); });
      const LoadMap lm = load_map(g.C, g.N, Np);
      add("mix.A_log", {C, N}, [=](const void* s, int dt, hipStream_t st) -> int {
        TRY(h_load_nk(s, dt, a2, lm, st));
        hipLaunchKernelGGL(k_scan_rates, dim3((unsigned)((C * Np + 255) / 256)), dim3(256), 0, st, a2, (int)C, (int)N, Np);
        LAUNCHCHK();
        return IXT_OK;
      });
    }
    TRY(h_mat(c, &L.o, g.C, E));
    mat("mix.o", L.o, E, g.C, 0);
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
      m->tensors[p + n] = HTensor{m->norm_kind == IXT_NORM_ONE ? std::vector<int64_t>{} : std::vector<int64_t>{E}, nullptr, true};
      if (m->norm_kind == IXT_NORM_TANH) m->tensors[p + n + ".alpha"] = HTensor{{}, nullptr, true};
      if (m->norm_kind == IXT_NORM_TANH || m->norm_kind == IXT_NORM_LAYER) m->tensors[p + n + ".b"] = HTensor{{E}, nullptr, true};
    }
    return IXT_OK;
  }
  TRY(norm("norm2", m->norm_places & IXT_NORM_BEFORE ? &L.n2 : &L.n2b));
  if (both) TRY(norm("norm2b", &L.n2b));
  const bool gated = l.glu < IXT_ACT_RELU2;
  auto unit = [&](const std::string& q, const HMat& gu, const HMat& down, int ff, size_t gu_off = 0, size_t down_off = 0) {
    if (gated) {
      LoadMap gate = load_map(ff, E, gu.Kp), up = load_map(ff, E, gu.Kp, 1);
      gate.inter = up.inter = 1;
      mat_as(q + "gate", gu, gate, gu_off);
      mat_as(q + "up", gu, up, gu_off);
    } else mat_as(q + "up", gu, load_map(ff, E, gu.Kp), gu_off);
    mat_as(q + "down", down, load_map(E, ff, down.Kp), down_off);
  };
  const bool moe = l.ffn == IXT_FFN_MOE;
  const int n = moe ? l.experts : 1;
  TRY(h_mat(c, &L.gu, E, (gated ? 2 : 1) * up_to(l.ff, IXT_KALIGN), n));
  TRY(h_mat(c, &L.down, l.ff, E, n));
  L.gu_stride = (size_t)L.gu.Kp * L.gu.Np; L.down_stride = (size_t)L.down.Kp * L.down.Np;
  for (int e = 0; e < n; ++e) unit(moe ? "mlp.e" + std::to_string(e) + "." : "mlp.", L.gu, L.down, l.ff, e * L.gu_stride, e * L.down_stride);
  if (l.glu == IXT_ACT_XIELU) {
    TRY(h_allocf(c, &L.unit, 4)); TRY(h_allocf(c, &L.unit_par, 4));
    float *d = L.unit, *par = L.unit_par;
    add("mlp.act", {2}, [=](const void* s, int dt, hipStream_t st) -> int {
      TRY(h_load_vec(s, dt, d, (int64_t)2, st));
      hipLaunchKernelGGL(k_xielu_numbers, dim3(1), dim3(64), 0, st, d, par);
      LAUNCHCHK();
      return IXT_OK;
    });
  }
  if (!moe) return IXT_OK;
  if (l.shared_ff > 0) {
    TRY(h_mat(c, &L.sgu, E, (gated ? 2 : 1) * up_to(l.shared_ff, IXT_KALIGN)));
    TRY(h_mat(c, &L.sdown, l.shared_ff, E));
    unit("mlp.shared.", L.sgu, L.sdown, l.shared_ff);
  }
  const bool sg = l.shared_ff > 0 && l.shared_gate;
  TRY(h_allocf(c, &L.router, (size_t)(l.experts + sg) * m->Ep));
  float* d = L.router;
  if (sg) {                                                       // one more row behind the experts
    float* dg = d + (size_t)l.experts * m->Ep;
    const LoadMap lg = load_map(1, E, m->Ep);
    add("mlp.shared.sg", {1, E}, [=](const void* s, int dt, hipStream_t st) { return h_load_nk(s, dt, dg, lg, st); });
  }
  if (l.router_bias) TRY(vec("mlp.router.b", &L.bias, l.experts, {l.experts}));
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
  m->norm_kind = cf.norm_kind; m->norm_places = cf.norm_places; m->streams = cf.streams; m->tied = cf.logits_via_embedding != 0; m->logit_scale = cf.logit_scale;
  const int n = cf.num_decoder_layers, R = c->Rmax, Rp = up_to(R, 128);
  m->layers.resize(n);
  TRY(h_alloc(c, &m->embed, (size_t)m->V * m->E * m->esz));
  TRY(h_mat(c, &m->head, m->E, m->V));
  { void *d = m->embed, *dh = m->head.w; const int64_t ne = (int64_t)m->V * m->E; const bool f = m->f32, tied = m->tied; const LoadMap lm = load_map(m->V, m->E, m->head.Kp);
    auto head = [=](const void* s, int dt, hipStream_t st) { return h_load_mat(m, s, dt, dh, lm, st); };
    m->tensors["embed"] = HTensor{{m->V, m->E}, [=](const void* s, int dt, hipStream_t st) -> int {
      if (tied) TRY(head(s, dt, st));                              // (twice in memory: rows for the lookup, the dot's order for the logits)
      return f ? h_load_vec(s, dt, (float*)d, ne, st) : h_load_vec(s, dt, (bf16_t*)d, ne, st);
    }, false};
    if (!tied) m->tensors["head"] = HTensor{{m->V, m->E}, head, false}; }
  TRY(hybrid_norm_params(c, "final.norm", &m->fnorm));
  std::map<std::vector<float>, std::pair<float*, float*>> ropes;
  size_t act_k = m->Ep, hact_k = 0, qx_e = 0, qr_e = 0, olat_e = 0, part = 0, part2 = 0, s_q = 0, s_kq = 0, s_v = 0, s_dec = 0, s_b = 0, xg_e = 0, mh_e = 0, mi = 0, po = 0, ret_u = 0, part3 = 0, scan_t = 0, scan_u = 0, scan_s = 0;
  bool shifts = false;
  const size_t max_chunks = (size_t)R / SEG_CHUNK + (size_t)std::min(R, c->G) + 1;      // of a pass: a group has at most one run of rows
  auto upd = [](size_t& a, size_t v) { if (v > a) a = v; };
  // f32 slices of a dot over at most R rows (split-K only below 128 rows; launch_dot keeps to one slice when the slices do not fit)
  auto dot_floats = [&](int K, int N) { return std::max((size_t)R * N, (size_t)std::min(R, 128) * N * ((K + IXT_CHAIN - 1) / IXT_CHAIN)); };
  auto dotsz = [&](int K, int N) { upd(part, dot_floats(K, N)); };
  // a mixer of columns c0 .. of the input projection and rows oc .. of the output projection: its geometry, caches and states
  auto columns = [&](HLayer& L, int i, int c0, int oc) -> int {
    const ixt_layer& l = L.c;
    L.c0 = c0;
    if (l.mixer == IXT_MIX_ATTENTION) {
      HeadsGeom& g = L.hg;
      g.H = l.heads; g.G = l.kv_heads; g.d = l.dim; g.dv = l.vdim; g.rot = l.rot_dim; g.P = c->P; g.mpg = c->mpg; g.window = l.window; g.chunk = std::max(l.chunk, 0); g.scale = l.attn_scale;
      g.maps = std::max(l.maps, 1); g.cap = l.softcap; g.head_gate = l.out_gate == 2; g.oc = oc; g.of = l.mix_scale;
      if (!heads_mfma_sizes(l.dim, g.maps, l.vdim, m->f32, &g.dkp, &g.dvp)) { g.dkp = g.maps * up_to(l.dim, 32); g.dvp = up_to(l.vdim, 32); }
      g.dmp = g.dkp / g.maps;
      g.hs = up_to(l.dim, 4); g.vs = up_to(l.vdim, 4); g.ok = up_to(g.H * g.maps * g.hs, 16);
      g.ov = l.key_values ? g.ok : g.ok + up_to(g.G * g.maps * g.hs, 16);
      g.og = l.out_gate ? g.ov + up_to(g.G * g.vs, 16) : -1;
      L.in_cols = g.og >= 0 ? g.og + (g.head_gate ? g.H : g.H * g.vs) : g.ov + g.G * g.vs;
      L.o_rows = g.H * g.vs;
      const size_t tokens = (size_t)cf.pagedattn_num_pages * c->P * g.G;
      if (tokens > (size_t)INT32_MAX) return set_err(IXT_ERR_UNSUPPORTED, "layer %d: %zu cached heads in the page pool", i, tokens);
      TRY(h_alloc(c, &L.pages, tokens * g.dkp * m->esz));
      TRY(h_alloc(c, &L.vpages, tokens * g.dvp * m->esz));
      upd(qx_e, (size_t)R * g.H * g.dkp);
      upd(po, (size_t)IXT_HEADS_SPLIT_BLOCKS * 16 * g.dvp);
    } else {
      m->recurrent = true;
      RetGeom& g = L.rg;
      g.H = l.heads; g.d = l.dim; g.dv = l.vdim; g.dp = up_to(l.dim, 16); g.dvp = up_to(l.vdim, 16); g.rot = l.rot_dim;
      g.hs = up_to(l.dim, 4); g.vs = up_to(l.vdim, 4);
      g.ok = up_to(g.H * g.hs, 16); g.ov = 2 * g.ok; g.og = g.ov + up_to(g.H * g.vs, 16);
      g.silu = g.join_norm = l.mixer == IXT_MIX_LIGHTNING; g.kf = g.silu ? 1.0f : (float)(1.0 / sqrt((double)l.dim)); g.oc = oc; g.of = l.mix_scale;
      L.in_cols = g.og + g.H * g.vs;
      L.o_rows = g.H * g.vs;
      TRY(h_allocf(c, &L.state, (size_t)c->G * g.H * g.dp * g.dvp));
      std::vector<float> pw((size_t)g.H * (SEG_CHUNK + 1));
      for (int h = 0; h < g.H; ++h)
        for (int j = 0; j <= SEG_CHUNK; ++j) pw[(size_t)h * (SEG_CHUNK + 1) + j] = (float)pow(l.decay[h], j);
      TRY(h_allocf(c, &L.pow, pw.size()));
      HIPCHK(hipMemcpy(L.pow, pw.data(), pw.size() * 4, hipMemcpyHostToDevice));
      upd(s_q, (size_t)R * g.H * g.dp); upd(s_v, (size_t)R * g.H * g.dvp); upd(ret_u, max_chunks * g.H * g.dp * g.dvp);
    }
    return hybrid_rope(c, l, &ropes, &L);
  };
  for (int i = 0; i < n; ++i) {
    HLayer& L = m->layers[i];
    L.c = cf.layers[i];
    L.src = L.c.weights_of >= 0 ? L.c.weights_of : i;
    const ixt_layer& l = L.c;
    if (l.shift) {
      shifts = m->recurrent = true;
      TRY(h_allocf(c, &L.shift, (size_t)c->G * 2 * m->Ep));
    }
    m->passes = std::max(m->passes, l.loop_pass + 1);
    if (l.mixer == IXT_MIX_LATENT_ATTENTION) {
      LatentGeom& g = L.lg;
      g.H = l.heads; g.dn = l.dim; g.dr = l.rot_dim; g.rank = l.kv_rank; g.P = c->P; g.mpg = c->mpg; g.window = l.window; g.scale = l.attn_scale;
      g.rankp = latent_rankp(l.kv_rank); g.rotp = latent_rotp(l.rot_dim);
      const int NQ = up_to(g.H * (g.dn + g.dr), 16);
      L.d_off = l.q_rank > 0 ? up_to(l.q_rank, 16) : NQ;
      L.g_off = L.d_off + up_to(g.rank + g.dr, 16);
      TRY(h_alloc(c, &L.pages, (size_t)cf.pagedattn_num_pages * c->P * (g.rankp + g.rotp) * m->esz));
      TRY(hybrid_rope(c, l, &ropes, &L));
      m->maxH = std::max(m->maxH, g.H);
      const int dnp = up_to(g.dn, IXT_KALIGN), ukn = up_to(g.rankp, 16), kp = up_to(g.rankp, IXT_KALIGN), uvn = up_to(l.vdim, 16);
      {                                                                     // (with a query latent or a gate it stays in use beside the dots behind it)
        const int N = up_to(l.out_gate ? L.g_off + g.H * l.vdim : L.d_off + g.rank + g.dr, 16);
        dotsz(m->Ep, N);
        if (l.out_gate || l.q_rank > 0) upd(part2, std::max((size_t)R * N, (size_t)std::min(R, 128) * N * ((m->Ep + IXT_CHAIN - 1) / IXT_CHAIN)));
        if (l.q_rank > 0) { dotsz(up_to(l.q_rank, IXT_KALIGN), NQ); upd(act_k, up_to(l.q_rank, IXT_KALIGN)); }
      }
      upd(part, (size_t)g.H * Rp * ukn);                                    // several slices only below 128 rows
      upd(part, (size_t)g.H * up_to(std::min(R, 128), 16) * ukn * ((dnp + IXT_CHAIN - 1) / IXT_CHAIN));
      upd(part, (size_t)g.H * Rp * uvn);
      upd(part, (size_t)g.H * up_to(std::min(R, 128), 16) * uvn * ((kp + IXT_CHAIN - 1) / IXT_CHAIN));
      dotsz(up_to(g.H * l.vdim, IXT_KALIGN), up_to(m->E, 16));
      upd(act_k, up_to(g.H * l.vdim, IXT_KALIGN));
      upd(qx_e, (size_t)g.H * Rp * dnp); upd(qr_e, (size_t)R * g.H * g.rotp); upd(olat_e, (size_t)g.H * Rp * kp);
      upd(po, (size_t)(1024 + g.H) * 16 * g.rankp);
    } else if (column_mixer(l)) {
      TRY(columns(L, i, 0, 0));
      int n_in = L.in_cols, n_o = L.o_rows;
      if (l.beside) {
        L.side = std::make_unique<HLayer>();
        L.side->c = *l.beside; L.side->src = L.src;
        TRY(columns(*L.side, i, up_to(n_in, 16), n_o));
        n_in = up_to(n_in, 16) + L.side->in_cols; n_o += L.side->o_rows;
      }
      L.in_cols = n_in; L.okp = up_to(n_o, IXT_KALIGN);
      (L.c.mixer == IXT_MIX_ATTENTION ? L.hg.kend : L.rg.kend) = L.side ? L.o_rows : L.okp;
      if (L.side) { L.side->okp = L.okp; (L.side->c.mixer == IXT_MIX_ATTENTION ? L.side->hg.kend : L.side->rg.kend) = L.okp; }
      L.o_rows = n_o;
      dotsz(m->Ep, up_to(n_in, 16));
      dotsz(L.okp, up_to(m->E, 16));
      upd(act_k, L.okp);
    } else if (l.mixer == IXT_MIX_SCAN) {
      m->recurrent = true;
      ScanGeom& g = L.sg;
      g.C = l.inner; g.Cp = up_to(l.inner, 4); g.N = l.state; g.rank = l.dt_rank; g.taps = l.conv;
      for (g.Np = 16; g.Np < g.N;) g.Np *= 2;
      g.oz = up_to(g.C, 16); g.ob = up_to(g.rank, 16); g.oc = g.ob + up_to(g.N, 16);
      L.okp = up_to(g.C, IXT_KALIGN);
      TRY(h_allocf(c, &L.state, (size_t)c->G * g.C * g.Np));
      TRY(h_allocf(c, &L.tails, (size_t)c->G * 2 * (g.taps - 1) * g.Cp + 4));
      const int Nx = up_to(g.oc + g.N, 16), Nd = up_to(g.C, 16), Kd = up_to(g.rank, IXT_KALIGN);
      dotsz(m->Ep, up_to(g.oz + g.C, 16));
      upd(part2, std::max((size_t)R * Nx, (size_t)std::min(R, 256) * Nx * ((L.okp + IXT_CHAIN - 1) / IXT_CHAIN))); upd(part3, dot_floats(Kd, Nd));
      dotsz(L.okp, up_to(m->E, 16));
      upd(act_k, L.okp);
      upd(scan_t, (size_t)Rp * Kd); upd(scan_u, max_chunks * g.C * g.Np); upd(scan_s, max_chunks * g.Cp);
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
  if (shifts && !m->h32) TRY(h_allocf(c, &m->h32, (size_t)R * m->E));
  if (m->passes > 0) {
    TRY(h_mat(c, &m->loop_in, 2 * m->Ep, m->E)); TRY(h_allocf(c, &m->loop_step, (size_t)m->passes * m->Ep)); TRY(h_alloc(c, &m->cat, (size_t)Rp * 2 * m->Ep * m->esz));
    dotsz(2 * m->Ep, up_to(m->E, 16));
    LoadMap lm = load_map(m->E, 2 * m->E, m->loop_in.Kp);
    lm.kg = m->E; lm.kgp = m->Ep;
    void* d = m->loop_in.w;
    m->tensors["loop.in"] = HTensor{{m->E, 2 * (int64_t)m->E}, [=](const void* s, int dt, hipStream_t st) { return h_load_mat(m, s, dt, d, lm, st); }, false};
    const LoadMap ls = load_map(m->passes, m->E, m->Ep);
    float* step = m->loop_step;
    m->tensors["loop.step"] = HTensor{{m->passes, m->E}, [=](const void* s, int dt, hipStream_t st) { return h_load_nk(s, dt, step, ls, st); }, false};
  }
  for (int i = 0; i < n; ++i) {
    if (m->layers[i].src == i) TRY(hybrid_layer_params(c, i));
    m->layers[i].c.beside = nullptr;               // (the caller's array may go)
  }
  m->missing = 0;
  for (auto& kv : m->tensors) m->missing += kv.second.done ? 0 : 1;
  upd(part, (size_t)c->NLmax * m->head.Np * (c->NLmax < 128 ? (m->head.Kp + IXT_CHAIN - 1) / IXT_CHAIN : 1));
  c->part_floats = part; TRY(h_allocf(c, &c->part, part));
  m->part2_floats = part2; TRY(h_allocf(c, &m->part2, part2 + 4));
  m->part3_floats = part3; TRY(h_allocf(c, &m->part3, part3 + 4));
  TRY(h_alloc(c, &m->scan_t, (scan_t + 8) * m->esz)); TRY(h_allocf(c, &m->scan_u, scan_u + 4)); TRY(h_allocf(c, &m->scan_sum, scan_s + 4));
  TRY(h_allocf(c, &m->x, (size_t)R * std::max(1, m->streams) * m->E));
  TRY(h_allocf(c, &m->ret_u, ret_u + 4)); TRY(h_allocf(c, &m->chunk, max_chunks)); TRY(h_allocf(c, &m->sgate, (size_t)R + 4));
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
  auto state = [&](float* p, int64_t floats) { sb.push_back(p); sp.push_back(floats); };
  auto pool = [&](void* p, int64_t elems) { pp.push_back((char*)p); pb.push_back(elems * (int64_t)m->esz); };
  auto group = [&](const HLayer& L) {
    if (L.c.mixer == IXT_MIX_ATTENTION) { pool(L.pages, (int64_t)c->P * L.hg.G * L.hg.dkp); pool(L.vpages, (int64_t)c->P * L.hg.G * L.hg.dvp); }
    else if (L.c.mixer == IXT_MIX_LATENT_ATTENTION) pool(L.pages, (int64_t)c->P * (L.lg.rankp + L.lg.rotp));
    else if (L.c.mixer == IXT_MIX_RETENTION || L.c.mixer == IXT_MIX_LIGHTNING) state(L.state, (int64_t)L.rg.H * L.rg.dp * L.rg.dvp);
    else if (L.c.mixer == IXT_MIX_SCAN) { state(L.state, (int64_t)L.sg.C * L.sg.Np); state(L.tails, (int64_t)2 * (L.sg.taps - 1) * L.sg.Cp); }
    else { state(L.state, (int64_t)L.dg.H * L.dg.dv * L.dg.dp); state(L.tails, (int64_t)2 * (L.dg.taps - 1) * L.dg.C); }
    if (L.shift) state(L.shift, (int64_t)2 * m->Ep);
  };
  for (const HLayer& L : m->layers) { group(L); if (L.side) group(*L.side); }
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
// a product of few columns over a long K, some rows: whole-K blocks would leave most of the chip idle, so the reduction is cut into slices (128 x 160 outputs, K
// 4096: 7 against 16 us; from 1024 rows on the whole form is as fast)
template <typename T> static int hdot_narrow(ixt_ctx* c, const T* x, const HMat& w, int R, float* out, size_t out_floats, hipStream_t st, Slices* res) {
  if constexpr (sizeof(T) == 2) {
    const int chains = (w.Kp + IXT_CHAIN - 1) / IXT_CHAIN;
    if (R >= c->ring_min_rows && R <= 256 && chains >= 4 && (w.Np + 31) / 32 * ((R + 63) / 64) <= 96 && (size_t)chains * R * w.Np <= out_floats) {
      DotResult dr;
      TRY(launch_dot(c, x, (const bf16_t*)w.w, w.Kp, w.Np, R, out, out_floats, false, st, &dr, true));
      *res = Slices{out, dr.slices, dr.slice_stride, w.Np};
      return IXT_OK;
    }
  }
  return hdot<T>(c, x, w, R, out, out_floats, st, res);
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
// product with a unit without a gate (from IXT_ACT_RELU2 on) behind it -> act(T) of the down product
template <typename T> static int hact_unit(ixt_ctx* c, const T* x, const HMat& w, size_t stride, int rows, int group_rows, const int32_t* rb, int kind, const float* par, T* out, hipStream_t st);
template <> int hact_unit<bf16_t>(ixt_ctx* c, const bf16_t* x, const HMat& w, size_t stride, int rows, int group_rows, const int32_t* rb, int kind, const float* par, bf16_t* out, hipStream_t st) {
  GemmEpi e{};
  e.act = out; e.glu = kind; e.act_par = par; e.rb_exp = rb; e.wstride = stride / 8;
  if (rb ? group_rows % 128 == 0 : rows >= c->ring_min_rows) return launch_ring(c, GEPI_ACT, x, (const bf16_t*)w.w, w.Kp, w.Np, rows, e, false, st);
  if (!rb && rows <= c->small_rows && sdot_plan(c, GEPI_ACT, false, w.Kp, w.Np, rows).ok) return launch_sdot(c, GEPI_ACT, false, x, nullptr, (const bf16_t*)w.w, w.Kp, w.Np, rows, e, st);
  const int rowblocks = (rows + 15) / 16, nrb = rb ? 1 : (rowblocks >= 3 ? 4 : rowblocks), zblocks = (rowblocks + nrb - 1) / nrb, ntile = w.Np / 16;
  dim3 grid((((ntile + 3) / 4 + 7) / 8) * 8 * zblocks, 1, 1);
#define HACT(B_, NT_) hipLaunchKernelGGL((k_dotb<B_, false, NT_, 2>), grid, dim3(256), (size_t)(B_) * 16 * 1024, st, reinterpret_cast<const u32x4*>(x), reinterpret_cast<const u32x4*>(w.w), \
                                         w.Kp, w.Np, rows, reinterpret_cast<float*>(out), ntile, zblocks, rb, stride / 8, kind, 0.0f, par)
  if (nrb == 4) { if (zblocks == 1) HACT(4, true); else HACT(4, false); }
  else if (nrb == 2) HACT(2, true);
  else HACT(1, true);
#undef HACT
  LAUNCHCHK();
  return IXT_OK;
}
template <> int hact_unit<float>(ixt_ctx* c, const float* x, const HMat& w, size_t stride, int rows, int, const int32_t* rb, int kind, const float* par, float* out, hipStream_t st) {
  Slices t;
  TRY(hdot_grouped<float>(c, x, w, stride, rows, 16, rb, c->part, c->part_floats, st, &t));
  hipLaunchKernelGGL((k_act_slices<float>), dim3(rows, (w.Np + 255) / 256), dim3(256), 0, st, t, w.Np, kind, par, out, rb);
  LAUNCHCHK();
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
  Slices t, in;
  const bool kept = L.c.out_gate || L.c.q_rank > 0;              // the input projection outlives the next dots
  TRY(hdot<T>(c, (const T*)m->xb, W.in, R, kept ? m->part2 : c->part, kept ? m->part2_floats : c->part_floats, st, &in));
  t = in;
  if (L.c.q_rank > 0) {
    hipLaunchKernelGGL((k_rms_x<T>), dim3(R), dim3(256), 0, st, in, 0, L.c.q_rank, W.qnorm, m->eps, (T*)m->act, W.uq.Kp);
    LAUNCHCHK();
    TRY(hdot<T>(c, (const T*)m->act, W.uq, R, c->part, c->part_floats, st, &t));
  }
  hipLaunchKernelGGL((k_latent_prep<T>), dim3(R, 1 + (g.H + 3) / 4), dim3(256), 0, st, in, t, L.d_off, g, W.cnorm, m->eps, L.rope_cos, L.rope_sin, c->row_slot, c->row_pos, c->row_active,
                     c->ps.page_map, (T*)L.pages, (T*)m->qx, W.uk.Kp, Rp, (T*)m->qr);
  LAUNCHCHK();
  TRY(hdot_grouped<T>(c, (const T*)m->qx, W.uk, W.uk_stride, g.H * Rp, Rp, m->head_rb, c->part, c->part_floats, st, &t));
  TRY(latent_attention<T>(c, L, t, R, Rp, decode, len_hint, st));
  TRY(hdot_grouped<T>(c, (const T*)m->olat, W.uv, W.uv_stride, g.H * Rp, Rp, m->head_rb, c->part, c->part_floats, st, &t));
  hipLaunchKernelGGL((k_heads_x<T>), dim3(R, (W.o.Kp + 255) / 256), dim3(256), 0, st, t, g.H, L.c.vdim, Rp, L.c.out_gate ? in : Slices{}, L.g_off, (T*)m->act, W.o.Kp);
  LAUNCHCHK();
  return IXT_OK;
}

// one mixer, or two side by side, on columns of one projection
template <typename T>
static int hybrid_mixer_columns(ixt_ctx* c, const HLayer& L, const HLayer& W, int R, int nseg_max, bool decode, int len_hint, hipStream_t st) {
  Slices t;
  TRY(hdot<T>(c, (const T*)c->hy->xb, W.in, R, c->part, c->part_floats, st, &t));
  t.bias = W.ibias;
  auto one = [&](const HLayer& l, const HLayer& w, const Slices& own) -> int {
    if (l.c.mixer == IXT_MIX_ATTENTION) return heads_attention<T>(c, l, w, own, R, decode, len_hint, st);
    return retention_mix<T>(c, l, w, own, R, nseg_max, decode, st);
  };
  bool done = false;
  if (decode) TRY(heads_beside_retention<T>(c, L, W, t, R, len_hint, st, &done));
  if (done) return IXT_OK;
  TRY(one(L, W, t));
  return L.side ? one(*L.side, *W.side, t.from(L.side->c0)) : (int)IXT_OK;
}

template <typename T>
static int hybrid_mixer_scan(ixt_ctx* c, const HLayer& L, const HLayer& W, int R, int nseg_max, bool single, hipStream_t st) {
  HybridModel* m = c->hy;
  Slices in, low, dt{};
  TRY(hdot<T>(c, (const T*)m->xb, W.in, R, c->part, c->part_floats, st, &in));
  TRY(scan_conv<T>(c, L, W, in, R, st));
  TRY(hdot_narrow<T>(c, (const T*)m->act, W.low, R, m->part2, m->part2_floats, st, &low));
  if (!single || R > 32) {                                         // (few rows: k_scan_step works the step sizes out itself)
    TRY(scan_rank<T>(c, W, low, R, st));
    low.n = 1;
    TRY(hdot<T>(c, (const T*)m->scan_t, W.dt, R, m->part3, m->part3_floats, st, &dt));
    dt.bias = W.dtb;
  }
  return scan_mix<T>(c, L, W, in, low, dt, R, nseg_max, single, st);
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
  const RouteRule rule{l.experts, l.top, l.router, l.groups > 1 ? l.groups : 0, l.groups_keep, l.router_norm, l.router_scale, W.corr, W.bias, l.shared_ff > 0 && l.shared_gate ? m->sgate : nullptr};
  const bool gated = l.glu < IXT_ACT_RELU2;
  if (l.shared_ff > 0) {
    TRY(gated ? hglu<T>(c, (const T*)m->xb, W.sgu, 0, R, 0, nullptr, l.glu, l.glu_limit, (T*)m->hact, st) : hact_unit<T>(c, (const T*)m->xb, W.sgu, 0, R, 0, nullptr, l.glu, W.unit_par, (T*)m->hact, st));
    TRY(hdot<T>(c, (const T*)m->hact, W.sdown, R, m->part2, m->part2_floats, st, shared));
  }
  const float* h = (m->norm_places & IXT_NORM_BEFORE) ? m->h32 : m->x;
  const size_t lds = sizeof(float) * (l.experts + 2 * rule.groups);
  const int nw = n + (rule.gate != nullptr ? 1 : 0);              // rows of the router's matrix; 12 at a time where that saves a pass
#define HROUTE(NE_) do { \
    if (R <= 256) hipLaunchKernelGGL((k_route<1, NE_>), dim3(R), dim3(256), lds, st, h, W.router, m->E, m->Ep, rule, R, m->midx, m->mw); \
    else hipLaunchKernelGGL((k_route<4, NE_>), dim3((R + 3) / 4), dim3(256), 4 * lds, st, h, W.router, m->E, m->Ep, rule, R, m->midx, m->mw); \
  } while (0)
  if ((nw + 11) / 12 < (nw + 7) / 8) HROUTE(12); else HROUTE(8);
#undef HROUTE
  LAUNCHCHK();
  const int align = (m->f32 || pairs <= 64) ? 16 : 128;
  const int rows_g = up_to(pairs, align) + align * std::min(n, pairs);     // every expert with a copy may waste up to align - 1 rows
  if (rows_g > m->moe_cap) return set_err(IXT_ERR_INVALID, "moe: %d copies exceed the routed workspaces", pairs);
  hipLaunchKernelGGL(k_moe_plan_any, dim3(1), dim3(1024), 0, st, m->midx, pairs, n, align, rows_g / 16, m->mpos, m->mrb);
  if constexpr (sizeof(T) == 2) hipLaunchKernelGGL(k_moe_gather, dim3(pairs, (m->Ep + 2047) / 2048), dim3(256), 0, st, (const bf16_t*)m->xb, m->mpos, l.top, m->Ep, (bf16_t*)m->xg);
  else hipLaunchKernelGGL(k_gather32, dim3(pairs, (m->Ep + 255) / 256), dim3(256), 0, st, (const float*)m->xb, m->mpos, l.top, m->Ep, (float*)m->xg);
  LAUNCHCHK();
  TRY(gated ? hglu<T>(c, (const T*)m->xg, W.gu, W.gu_stride, rows_g, align, m->mrb, l.glu, l.glu_limit, (T*)m->mhact, st)
            : hact_unit<T>(c, (const T*)m->xg, W.gu, W.gu_stride, rows_g, align, m->mrb, l.glu, W.unit_par, (T*)m->mhact, st));
  return hdot_grouped<T>(c, (const T*)m->mhact, W.down, W.down_stride, rows_g, align, m->mrb, c->part, c->part_floats, st, out);
}

// logits of rows lrows[i] (or lrow0 + i) of the residual stream, NLmax at a time
template <typename T>
static int hybrid_logits(ixt_ctx* c, int R, int lrow0, int nl, const int32_t* lrows, int32_t* argmax_out, float* logits_out, hipStream_t st) {
  HybridModel* m = c->hy;
  const int nblk = (m->V + 1023) / 1024;
  for (int i0 = 0; i0 < nl; i0 += c->NLmax) {
    const int n = std::min(c->NLmax, nl - i0);
    TRY((hybrid_final_norm<T>(c, R, n, lrows ? lrows + i0 : nullptr, lrow0 + i0, st)));
    Slices t;
    TRY(hdot<T>(c, (const T*)m->xn, m->head, n, c->part, c->part_floats, st, &t));
    hipLaunchKernelGGL(k_head_post, dim3(nblk, n), dim3(256), 0, st, t, m->V, m->logit_scale, c->sample_cols, logits_out ? logits_out + (size_t)i0 * m->V : nullptr, c->amax_val, c->amax_idx);
    if (argmax_out) hipLaunchKernelGGL(k_argmax_final, dim3(n), dim3(256), 0, st, c->amax_val, c->amax_idx, nblk, argmax_out + i0);
    LAUNCHCHK();
  }
  return IXT_OK;
}

// a sublayer's last product and what follows it: x <- x + post(W v), the next operand pre(x).  Tanh norms ride in the product's epilogue where the whole
// sum is in one place.
template <typename T>
static int hybrid_dot_norm(ixt_ctx* c, const T* v, const HMat& w, const Around& ar, bool routed, int R, bool single, const float* bias, float fbias, hipStream_t st) {
  HybridModel* m = c->hy;
  [[maybe_unused]] const NormW &post = ar.post, &pre = ar.pre;
  if constexpr (sizeof(T) == 2) {
    const bool small = R <= c->small_rows && sdot_plan(c, GEPI_TANHNORM, false, w.Kp, w.Np, R).ok;
    if (m->norm_kind == IXT_NORM_TANH && m->streams == 0 && ar.mu == nullptr && !ar.to_cat && bias == nullptr && (small || R >= c->ring_min_rows)) {
      GemmEpi e{};
      e.act = (bf16_t*)m->xb;
      e.tn = TanhNormEpi{post.w, post.b, post.alpha, pre.w, pre.b, pre.alpha, m->x, routed && pre.w != nullptr ? m->h32 : nullptr, m->E, m->Ep};
      if (small) return launch_sdot(c, GEPI_TANHNORM, false, v, nullptr, (const bf16_t*)w.w, w.Kp, w.Np, R, e, st);
      return launch_ring(c, GEPI_TANHNORM, v, (const bf16_t*)w.w, w.Kp, w.Np, R, e, false, st);
    }
  }
  Slices t;
  TRY(hdot<T>(c, v, w, R, c->part, c->part_floats, st, &t));
  SubOut o{t};
  o.bias = bias; o.fbias = fbias;
  return hybrid_norm<T>(c, o, ar, routed, R, single, st);
}

template <typename T>
static int forward_rows_hybrid_t(ixt_ctx* c, int R, const int32_t* tokens, int len_hint, int lrow0, int nl, const int32_t* lrows, int32_t* argmax_out, float* logits_out, bool decode,
                                 int nseg_max, hipStream_t st) {
  HybridModel* m = c->hy;
  const int Rp = (sizeof(T) == 2 && R >= c->ring_min_rows) ? up_to(R, 128) : up_to(R, 16);
  if (m->recurrent || m->maxH > 0)
    hipLaunchKernelGGL(k_segments, dim3(1), dim3(1024), 0, st, R, c->row_active, c->row_slot, c->row_pos, m->row_seg, m->row_j, m->seg, m->chunk, m->nseg, m->state_len, m->parity, m->claim, c->G,
                     m->recurrent ? 1 : 0, m->err, m->head_rb, m->maxH * (Rp / 16), Rp / 16);
  const NormW none{};
  auto entry = [&](size_t i) {                                     // what stands in front of the mixer of run i
    const HLayer& W = m->layers[m->layers[i].src];
    return Around{none, W.n1, nullptr, W.hc1, W.mu, m->layers[i].shift, false};
  };
  auto before = [&](size_t i) {                                    // what a sublayer in front of run i leaves (the head's norm is taken of the wanted rows only)
    if (i >= m->layers.size()) return Around{none, none, nullptr, nullptr};
    if (m->layers[i].c.loop_pass >= 0) return Around{none, none, nullptr, nullptr, nullptr, nullptr, true};
    return entry(i);
  };
  const Around first = before(0);
  const bool tanh_first = m->norm_kind == IXT_NORM_TANH && m->streams == 0 && first.mu == nullptr;      // that norm rides with the lookup
  hipLaunchKernelGGL((k_embed_scaled<T>), dim3(R), dim3(256), 0, st, (const T*)m->embed, tokens, m->emb_scale, m->E, m->Ep, m->V, std::max(1, m->streams),
                     tanh_first ? first.pre : none, m->x, (T*)m->xb, (T*)m->cat);
  LAUNCHCHK();
  if (!tanh_first && (first.pre.w != nullptr || m->streams > 0)) TRY((hybrid_norm<T>(c, SubOut{}, first, false, R, decode, st)));
  for (size_t i = 0; i < m->layers.size(); ++i) {
    const HLayer& L = m->layers[i];
    const HLayer& W = m->layers[L.src];
    if (L.c.loop_pass >= 0) {                                      // a pass begins: x <- W [x; x0] + its step
      SubOut o{};
      TRY(hdot<T>(c, (const T*)m->cat, m->loop_in, R, c->part, c->part_floats, st, &o.t));
      o.bias = m->loop_step + (size_t)L.c.loop_pass * m->Ep; o.fresh = true;
      TRY((hybrid_norm<T>(c, o, entry(i), false, R, decode, st)));
    }
    if (L.c.mixer == IXT_MIX_LATENT_ATTENTION) TRY((hybrid_mixer_latent<T>(c, L, W, R, Rp, decode, len_hint, st)));
    else if (L.c.mixer == IXT_MIX_SCAN) TRY((hybrid_mixer_scan<T>(c, L, W, R, nseg_max, decode, st)));
    else if (column_mixer(L.c)) TRY((hybrid_mixer_columns<T>(c, L, W, R, nseg_max, decode, len_hint, st)));
    else TRY((hybrid_mixer_delta<T>(c, L, W, R, nseg_max, decode, st)));
    const bool ffn = L.c.ffn != IXT_FFN_NONE;
    Around ar1 = ffn ? Around{none, W.n2, nullptr, W.hc2} : before(i + 1), ar2 = before(i + 1);
    ar1.post = W.n1b; ar1.hc = W.hc1; ar2.post = W.n2b; ar2.hc = W.hc2;
    TRY((hybrid_dot_norm<T>(c, (const T*)m->act, W.o, ar1, L.c.ffn == IXT_FFN_MOE, R, decode, W.obias, L.c.mix_scale, st)));
    if (L.c.ffn == IXT_FFN_DENSE) {
      TRY(L.c.glu < IXT_ACT_RELU2 ? hglu<T>(c, (const T*)m->xb, W.gu, 0, R, 0, nullptr, L.c.glu, L.c.glu_limit, (T*)m->hact, st)
                                  : hact_unit<T>(c, (const T*)m->xb, W.gu, 0, R, 0, nullptr, L.c.glu, W.unit_par, (T*)m->hact, st));
      TRY((hybrid_dot_norm<T>(c, (const T*)m->hact, W.down, ar2, false, R, decode, nullptr, 1.0f, st)));
    } else if (L.c.ffn == IXT_FFN_MOE) {
      Slices t, shared{};
      const float* addw = L.c.shared_gate ? m->sgate : nullptr;
      TRY(hybrid_moe<T>(c, L, W, R, st, &t, &shared));
      if (t.n > 2 && R <= 64) {
        hipLaunchKernelGGL(k_moe_sum, dim3((t.ncols + 255) / 256, R), dim3(64), 0, st, t, m->mpos, m->mw, L.c.top, m->msum);
        LAUNCHCHK();
        TRY((hybrid_norm<T>(c, SubOut{Slices{m->msum, 1, 0, t.ncols}, shared, addw}, ar2, false, R, decode, st)));
      } else {
        TRY((hybrid_norm<T>(c, SubOut{t, shared, addw, m->mpos, m->mw, L.c.top}, ar2, false, R, decode, st)));
      }
    }
    if (m->tap && !c->capturing) {
      if ((i + 1) * (size_t)R * m->E > m->tap_floats) return set_err(IXT_ERR_INVALID, "residual tap: buffer too small");
      hipLaunchKernelGGL(k_stream_sum, dim3(R, (m->E + 255) / 256), dim3(256), 0, st, m->x, std::max(1, m->streams), m->E, m->tap + i * (size_t)R * m->E);
      LAUNCHCHK();
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
