// ixt_internal.h -- what the host objects of libixt share: the ctx, error reporting, memory ownership and the launch helpers of the canonical dot.
#pragma once
#include "../../include/ixt.h"
#include "ixt_kernels.h"

#include <hip/hip_runtime.h>
#include <math.h>
#include <stdint.h>
#include <string.h>

#include <algorithm>
#include <functional>
#include <map>
#include <string>
#include <vector>

int set_err(int code, const char* fmt, ...);
#define HIPCHK(expr)                                                                                   \
  do {                                                                                                 \
    hipError_t e_ = (expr);                                                                            \
    if (e_ != hipSuccess) return set_err(IXT_ERR_HIP, "%s failed: %s (%s:%d)", #expr, hipGetErrorString(e_), __FILE__, __LINE__); \
  } while (0)
#define LAUNCHCHK() HIPCHK(hipGetLastError())

struct LayerW {
  bf16_t *ln1, *wqkv, *wo, *ln2, *wi, *wout;
  bf16_t *pan = nullptr, *pfn = nullptr;   // Gemma-2 / 3: post-attention / post-MLP norm scales
  bf16_t *qn = nullptr, *kn = nullptr;     // Gemma-3: query / key head norm scales [head_dim]
  bf16_t* gate = nullptr;                  // Mixtral: MoeBlock_0/gate/kernel, row-major [emb][experts]
  std::vector<bf16_t*> ewi, ewout;         // Mixtral: per expert the (wi_0, wi_1) pair and wo in the dot kernels' layout (wi / wout unused)
};

enum { W_LN1 = 0, W_Q, W_K, W_V, W_O, W_LN2, W_WI0, W_WI1, W_WOUT, W_PER_LAYER, W_PAN = W_PER_LAYER, W_PFN, W_QN, W_KN, W_GATE };

struct TimingPair { hipEvent_t a, b; double bytes; int family; };   // family: 0 canonical dot (incl. unembedding), 1 one-launch decode attention

struct GraphEntry {
  hipGraphExec_t exec;
};

struct HybridModel;           // IXT_BLOCK_HYBRID (ixt_hybrid.h)
int hybrid_check(const ixt_config& c);
int hybrid_init(ixt_ctx* c);
int hybrid_load_weight(ixt_ctx* c, const std::string& name, const void* src, int dtype, const int64_t* shape, int ndim, hipStream_t st);
bool hybrid_complete(const ixt_ctx* c);
void hybrid_free(ixt_ctx* c);
HybridModel* hybrid_new();
int hybrid_copy_group(ixt_ctx* c, int src, int dst, int npages, hipStream_t st);
int hybrid_prompt_logits(ixt_ctx* c, int row0, int n, hipStream_t st);
int forward_rows_hybrid(ixt_ctx* c, int R, const int32_t* tokens, int len_hint, int lrow0, int nl, const int32_t* lrows, int32_t* argmax_out, float* logits_out, bool decode,
                               hipStream_t st);

struct ixt_ctx {
  ixt_config cfg;
  HybridModel* hy = nullptr;
  bool one_segment = false;    // the rows of the running call belong to one page group (ixt_prefill_chunk)
  int E, Q, KV, D, F, V, L, P, B, Rmax, NQKV, QN, KN, Tmax, mpg, nsb_max, GQ;
  int G = 0, S = 0;            // page groups = B decode slots + S staging groups of packed prefill
  int NLmax = 1;               // rows that can be unembedded in one call (decode slots / prompts of a packed prefill)
  // weights
  bf16_t* embedding = nullptr;
  bf16_t* final_norm = nullptr;
  bf16_t* logits_w = nullptr;
  std::vector<LayerW> layers;
  std::vector<uint32_t> loaded;  // per layer bitmask; index L = globals (bit0 emb, bit1 norm, bit2 logits)
  // tables / pools / state
  bf16_t *rope_sin = nullptr, *rope_cos = nullptr;
  bf16_t *rope_sin_local = nullptr, *rope_cos_local = nullptr;   // Gemma-3 local layers (local_rope_max_timescale); nullptr: the tables above
  std::vector<uint16_t> rope_sin_h, rope_cos_h;
  std::vector<float> rope_sin32_h, rope_cos32_h;   // rope_type "llama3.1": f32 tables; rope_sin / rope_cos then point at their device copies
  bool rope32 = false;
  std::vector<bf16_t*> kpages_l, vpages_l;   // one allocation per layer: [page][kv_head][...]
  bf16_t **kptrs_d = nullptr, **vptrs_d = nullptr;   // the same pointers in HBM (k_pages_copy)
  size_t layer_page_elems = 0;
  int32_t* lrows = nullptr;                  // rows to unembed (ixt_prefill_rows)
  PageStateDev ps{};
  // workspaces
  bf16_t *h_a = nullptr, *h_b = nullptr, *xn = nullptr, *qbuf = nullptr, *ao = nullptr, *hact = nullptr;
  float *part = nullptr, *scores = nullptr, *pvpart = nullptr, *amax_val = nullptr;
  int32_t* amax_idx = nullptr;
  size_t amax_cap = 0;
  bf16_t* xt_op = nullptr;  // op-level entry points: the caller's row-major x in the dot kernel's x layout
  size_t xt_cap = 0;
  bf16_t* wt_op = nullptr;  // ixt_op_dot: the caller's row-major kernel in the tiled weight layout (grown on demand)
  size_t wt_cap = 0;
  size_t part_floats = 0;
  int32_t *row_slot = nullptr, *row_pos = nullptr, *row_active = nullptr, *row_tok = nullptr, *new_tok = nullptr;
  AttnGeom geom{};
  // timing
  bool timing = false;
  int attn_fused_min_blocks = 64;    // (Mixtral-8x7B, 8 slots x 8 kv heads: one launch 19.5 ms per step against 20.5 for the split form)
  // tiled GEMM form of the dot: from 128 rows and 150 blocks of 128 x 128 (at C2 / 256 rows: the 2048 x 14336 MLP kernel only; the
  // 2048 x 6144 QKV kernel has 96 such blocks and measured slower than split-K, as did 64-column blocks)
  int gemm_min_rows = 128, gemm_min_blocks = 150;
  int gemm_prefix_halves = 0;   // measured at 256 rows on the MLP up-projection: decode step 5.39 vs 4.84 ms: off
  int gemm_split_min_blocks = 300;   // 128 x 128 x one-chain blocks (at C2 / 256 rows: the QKV and MLP-down kernels; +2.4 % end to end)
  int unembed_gemm = 1;
  // LDS-ring GEMM with fused epilogues (ixt_gemm.h) from this many rows; ring_cfg forces a tile (1: 128 x 128, 2: 128 x 64, 3: 64 x 32)
  int ring_min_rows = 128, ring_cfg = 0, ring_split = 0, ring_wlayout = 0;
  // MLP down-projection on the ring path: 1 = ring GEMM with the residual epilogue; 0 = split-K tiles (one f32 slice per 512-k chain, two blocks
  // per CU) + slice-sum / residual / norm kernel; -1 (default) = by shape: the ring form needs at least 192 whole-K blocks of 128 x 128 or 128 x 64
  int ring_down = -1;
  int unembed_tall = 1;      // 256 x 128 tiles for the unembedding at 129..256 rows (0: 128 x 128)
  int ring_two_per_cu = 1;   // ring GEMMs of >= 1024 rows: 32-k chunks in 4 slots (64 KiB of LDS), two blocks per CU
  int attn_tile = 1;         // prefill rows: tiled attention (k_attn_tile) from attn_tile_min_rows rows on
  int attn_tile_min_rows = 64;
  int attn_wave_pairs = 0;   // measured at 256 rows, 765 keys: 339 us per launch (4.7 TB/s) against 305 us (5.3 TB/s) for the block form
  // few rows (one row block): five launches per layer (ixt_small.h).  small_rows: most rows of that path (0: off); small_tpb: column tiles per
  // block of k_sdot (0: by shape); small_attn_waves: waves per (row, kv head) block of k_attn_small (4: k_attn_decode instead)
  int small_rows = 16, small_tpb = 0, small_attn_waves = 16, small_attn_max_blocks = 512;
  int dot_small = 0;         // ixt_op_dot through k_sdot where it fits (tests)
  // few rows: the keys of a (row, kv head) split over `S` blocks of k_attn_split (S = min(small_attn_split, 256 / (rows * kv heads)); < 2: k_attn_small)
  int small_attn_split = 16;
  int split_capacity = -1;   // blocks of k_attn_split the chip holds at once (occupancy query, once)
  int moe_mid_pairs = 0;     // routed experts: up to this many (row, expert) copies per launch take 64-row whole-K dots instead of the ring GEMM.  Measured SLOWER at Mixtral-8x7B's 256-token prefill (512 copies): 74.7 against 30.2 ms -- 4 waves per block cannot hide both operands' latency at 64 rows: off
  int moe_fused_gate = 1;    // routed experts at few copies: wi as whole-K blocks with the SwiGLU epilogue (0: split-K slices + k_swiglu_part)
  int gemma_tile = 1;        // Gemma blocks: tiled prefill attention (0: the per-row scores / PV / combine kernels)
  int moe_route_blocks = 1;  // router: one wave per 512-k block, all experts at once (0: one wave per expert)
  int32_t* split_cnt = nullptr;   // [16][KV][4] arrival counters (zero between launches) + the error word behind them
  float* split_ws = nullptr;      // [16][KV][split_stride]
  size_t split_stride = 0;
  int small_prefetch = 0;    // few-rows path: prefetch blocks stream the next launch's kernel into the Infinity Cache (ixt_prefetch).  Measured SLOWER (one utterance 1.19 against 1.03 ms per step, eight 1.33 against 1.23: a launch cannot end before its prefetch has, and an Infinity-Cache hit is only 1.4 x an HBM stream): off
  int small_prefetch_blocks = 64;
  int small_norm = 1;        // 1: the RMSNorm in front of the QKV / wi projections runs inside k_sdot; 0: k_rownorm launches (experiments)
  int dot_stream_min_blocks = 1 << 30;   // off: measured slower than split-K at 256 rows (decode 7.84 vs 7.68 ms/step, prefill 3.53 vs 3.31 ms)
  ColRanges sample_cols{};   // greedy sampling restricted to these columns (n == 0: all)
  // Gemma-2 block (ixt_config.decoder_block == 1): L counts (attention, MLP) sub-layers, two per reference layer (even: local sliding)
  bool gemma = false;
  bool moe = false;          // Mixtral (decoder_block == 3): the llama2 wiring with a routed mixture of NE expert MLPs, TK per row
  int NE = 1, TK = 1;
  int NEL = 1, E0 = 0;       // expert parallelism: this context's experts are E0 .. E0 + NEL - 1 (ixt_config.ep_rank / ep_size)
  int32_t* moe_idx = nullptr;   // [Rmax][TK]
  float* moe_w = nullptr;       // [Rmax][TK]
  bf16_t* moe_y = nullptr;      // [Rmax][TK][E]
  // routed evaluation (k_moe_plan / k_moe_gather, grouped k_dotb / k_gemm_ring): copies of a row sit in the rows of their expert
  int moe_grouped = 1;          // 0: every expert over all rows (round 2's form; experiments)
  int moe_rows_cap = 0;         // copy rows incl. alignment padding the workspaces hold
  int32_t* moe_pos = nullptr;   // [Rmax TK] destination row of every copy
  int32_t* moe_rbexp = nullptr; // [moe_rows_cap / 16] expert of every 16-row block, -1: none
  int32_t* moe_cnt = nullptr;   // [2 NE] counts, offsets
  bf16_t* moe_xg = nullptr;     // [moe_rows_cap][E] gathered inputs (xidx layout)
  bf16_t* moe_hact = nullptr;   // [moe_rows_cap][F] SwiGLU outputs (xidx layout)
  float* moe_comb = nullptr;    // [Rmax][E] the mixture as one f32 slice
  size_t moe_wi_stride = 0, moe_wo_stride = 0;   // elements between two experts' kernels
  bool gemma3 = false;       // Gemma-3 (decoder_block == 2): gemma = true as well; one sub-layer per layer, layer l local unless l % 6 == 5
  float pv_cap = 0.0f;       // soft cap / window of the attention launch being issued (k_attn_pv)
  int pv_window = 0;
  float* glogits = nullptr;  // [NLmax][V] logits rows when the caller asks for none (the cap and the sampling need them)
  // return_prompt_logp (ixt_prefill_prompt_logp): the hidden rows the last forward pass left behind, and a logits workspace made on first use
  const bf16_t* h_final = nullptr;
  int h_final_rows = 0;
  float* plogits = nullptr;     // [NLmax][V]
  int32_t* pargmax = nullptr;   // [NLmax]
  // IXT-FP8-v1 (ixt_fp8.h): e4m3 twin + column scales of every projection kernel (made from the bf16 copy on first use), activation workspace
  struct F8W { uint8_t* w8; float* s; int K, N; };
  bool fp8 = false, fp8_ready = false;
  std::map<const bf16_t*, F8W> f8w;
  uint8_t* x8 = nullptr;        // [rows16][Kmax] e4m3 fragments
  float* xs8 = nullptr;         // [rows16][chains]
  std::vector<TimingPair> tpairs;
  size_t tused = 0;
  // graphs keyed by the pointer tuple of ixt_generate
  std::map<std::string, GraphEntry> graphs;
  bool capturing = false;
  std::vector<void*> allocs;
};

template <typename T>
static int dmalloc(ixt_ctx* c, T** p, size_t n) {
  void* q = nullptr;
  HIPCHK(hipMalloc(&q, n * sizeof(T) + 256));
  c->allocs.push_back(q);
  *p = (T*)q;
  return IXT_OK;
}
#define TRY(x) do { int rc_ = (x); if (rc_ != IXT_OK) return rc_; } while (0)

// ---- launch helpers (ixt_api.hip)
struct DotResult { int slices; size_t slice_stride; int ntiles; };
struct SdotPlan { int chains, tpb, rpl; size_t lds; bool ok; int pf_blocks; };
int launch_ring(ixt_ctx* c, int epi, const bf16_t* x, const bf16_t* w, int K, int N, int R, const GemmEpi& e, bool split, hipStream_t st, int wring = 0, int* wave_cols = nullptr);
int launch_dot(ixt_ctx* c, const bf16_t* x, const bf16_t* w, int K, int N, int R, float* out, size_t out_floats, bool force_full, hipStream_t st, DotResult* res, bool no_ring = false);
SdotPlan sdot_plan(const ixt_ctx* c, int epi, bool norm, int K, int N, int R);
int launch_sdot(ixt_ctx* c, int epi, bool norm, const bf16_t* x, const bf16_t* scale, const bf16_t* w, int K, int N, int R, const GemmEpi& e, hipStream_t st,
                const bf16_t* pf = nullptr, size_t pf_elems = 0);
