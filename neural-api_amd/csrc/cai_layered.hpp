// Declarations shared by the layered-decoder translation units: 16-bit weights, paged cache and state slots, recurrent mixers (the
// gated delta rule, state-space duality, forget-gate linear attention), attention over pages (keys and values, or one latent for
// both), norms and input convolutions on the stream, mixtures of experts (gfx950 only).
#pragma once
#include "cai_internal.hpp"

namespace cai {

typedef __bf16 bf16_t;
typedef bf16_t bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

// Activations between two products are bfloat16 (the serving precision) or float (everything in 32-bit).
enum { ACT_T_BF16 = 0, ACT_T_F32 = 1 };
constexpr int LIN_PAD = 64;                 // widths of 16-bit matrices and of the activations they read are padded to this with zeros
inline int pad_to(int n, int m) { return (n + m - 1) / m * m; }

__device__ __forceinline__ float bf16_lo(uint32_t u) { return __builtin_bit_cast(float, u << 16); }
__device__ __forceinline__ float bf16_hi(uint32_t u) { return __builtin_bit_cast(float, u & 0xffff0000u); }
__device__ __forceinline__ uint16_t bf16_bits(float f) { return __builtin_bit_cast(uint16_t, (bf16_t)f); }
__device__ __forceinline__ float to_f32(float v) { return v; }
__device__ __forceinline__ float to_f32(bf16_t v) { return (float)v; }

// Dynamic Tanh: y = w * tanh(alpha x) + b.  No statistics, so it lives in the epilogue of whatever produces x.  w == null: none.
struct Dyt { const float* w = nullptr; const float* b = nullptr; float alpha = 0.0f; };
__device__ __forceinline__ float dyt(const Dyt& t, float x, int i) { return t.w ? tanhf(t.alpha * x) * t.w[i] + t.b[i] : x; }

// What a linear layer does with its finished sums.
enum { EPI_STORE = 0, EPI_GLU = 1, EPI_RESIDUAL = 2, EPI_SPLIT = 3, EPI_JOIN = 4 };
// activations of layered decoders only, beside the CAI_ACT_ ones: max(v, 0)^2;  limit * tanh(v / limit)
constexpr int LIN_RELU_SQUARED = 100, LIN_SOFT_CAP = 101;
// Gated pairs: relu(g) u;  silu(g) u;  gelu(g) u, tanh form;  with g = min(gate, limit) and u = clamp(up, -limit, limit):
// g sigmoid(1.702 g) (u + 1)
enum { GLU_RELU = 0, GLU_SILU = 1, GLU_GELU_TANH = 2, GLU_CLAMPED = 3 };
struct LinEpi {
  int mode = EPI_STORE;
  float* y = nullptr; int64_t ldy = 0;              // STORE: result; RESIDUAL, JOIN: the residual stream, updated in place; SPLIT: the first results
  void* h = nullptr; int64_t ldh = 0;               // GLU: act(gate) * up; RESIDUAL: input of the next sublayer (null: none); SPLIT: the others
  const float* add0 = nullptr; int64_t ld0 = 0;     // RESIDUAL: added to the stream after the sum (start of a repeated pass)
  const float* bias = nullptr; int act = CAI_ACT_NONE;   // STORE: act(scale sum + bias); RESIDUAL: the sum includes it
  float scale = 1.0f;
  int split = 0;                                    // SPLIT: results [0, split) are sum + bias in y, the others act(sum + bias) in h
  const float* mult = nullptr; const float* gate = nullptr; int64_t ldg = 0;   // JOIN: y += mult[n] sigmoid(gate[t][n]) (sum + bias)
  int glu = GLU_RELU; float limit = 0.0f;           // limit: of GLU_CLAMPED and LIN_SOFT_CAP
  bool fresh = false;                               // RESIDUAL: x = post(sum) instead of x += post(sum)
  Dyt post, next;                                   // RESIDUAL: x += post(sum) [+ add0]; h = next(x)
};
// Gated matrices interleave their rows in blocks of 16: 16 gate rows, then the 16 up rows of the same outputs.
__host__ __device__ inline int glu_row(int j, int up) { return (j >> 4) * 32 + up * 16 + (j & 15); }

// y = W x for n_tok activation rows x[t][ldx] (zero padded to LIN_PAD columns, element type act_t); W is a CAI_BF16 matrix.
int launch_lin(const cai_qw_s* w, int act_t, const void* x, int64_t ldx, int n_tok, const LinEpi& e);
constexpr int LIN_FEW = 8;                  // up to so many rows take the streaming kernel
// Up to LIN_FEW rows of float columns x[t][ldx] through an RMS norm over the first `width` and a matrix, with one launch also through a second norm and
// matrix (null: none).  normed: where the normed rows themselves go, ldn apart and zero padded (null: nowhere; both ldn alike).
struct RmsLin { const cai_qw_s* w; const float* gain; LinEpi e; void* normed = nullptr; int64_t ldn = 0; };
int launch_lin_rms(int act_t, const float* x, int64_t ldx, int width, float eps, int n_tok, const RmsLin& a, const RmsLin* b);
// Up to LIN_FEW rows of two products with the same outputs that both join one stream.
int launch_lin_pair(int act_t, int n_tok, const cai_qw_s* w, const void* x, int64_t ldx, const LinEpi& e, const cai_qw_s* w2, const void* x2, int64_t ldx2, const LinEpi& e2);
// launch_lin over a bank of equal matrices stacked in w (mat_rows rows each): work lists of (matrix, first place, places) over an order
// of activation rows.  Place p reads activation row order[p] / div (div 0: row p) and writes row p of e.h, scaled by
// scale[order[p]] (GLU; SPLIT at 0: the activation of the sum), or row order[p] of e.y (STORE).
constexpr int BANK_TILE = 64, BANK_TILE_MAX = 128;      // most places of a list entry: one of the two
struct BankList { const int32_t *tiles, *n_tiles, *order; const float* scale; int div, tile, max_tiles; };   // tiles [.][3], n_tiles on the device
int launch_lin_bank(const cai_qw_s* w, int mat_rows, int act_t, const void* x, int64_t ldx, const BankList& l, const LinEpi& e);
// float columns [col0, col0 + cols) of x -> rows of the chosen type, zero padded to ldo
int launch_pack_rows(const float* x, int64_t ldx, int64_t col0, int cols, int n_tok, int act_t, void* out, int64_t ldo);
int bf16_dequant_rows(const cai_qw_s* w, int64_t row0, int64_t n_rows, float* out);
int bf16_linear_f32(const cai_qw_s* w, const float* x, int64_t ldx, int n_tok, float* y, int64_t ldy, int act);   // unpadded float rows in, float rows out
void bf16_release();

// ------------------------------------------------------------------------------------------
// Rows of one engine step.  A step is any number of entries (portions of prompts and single tokens) concatenated; per row the
// token, its position, the sequence slot and the first and last row of its entry; per entry slot, first row, rows, position.
// ------------------------------------------------------------------------------------------
struct StepRows {
  const int32_t *tok, *pos, *slot, *first, *last;   // [n_rows] device
  const int32_t* ent;                               // [n_ent][4] device: slot, row0, n, pos0
  int n_rows, n_ent;
  int reach;                                        // no position is this or more: what launches over the keys are sized by
};

// ------------------------------------------------------------------------------------------
// Paged key/value pool and recurrent-state slots.
// One page holds PAGE_TOKENS positions of every attention run (layer x pass) of ONE sequence; the pool is sized in tokens over
// all live sequences.  Page p of a sequence (positions p * PAGE_TOKENS ..) is table[slot][p mod ring]; pages that lie wholly
// before every window are handed back while the sequence runs on, so a ring of as many entries as the pool has pages never
// wraps onto a live page.  Recurrent state has one fixed place per (run, slot) and is read as zero at position 0.
// ------------------------------------------------------------------------------------------
constexpr int PAGE_TOKENS = 64;
struct AttnDims {
  int heads, kv_heads, dim, vdim, window; float scale, eps;
  int dim_p, vdim_p;                       // row strides in the pool: padded to 8 elements (zero filled)
  int chunked;                             // window is the size of fixed blocks of positions: a token sees its own block up to itself
  int rot; const double* turns;            // the first rot dimensions turn, i with i + rot / 2, by turns[i] full turns a position (0: none)
  int span;                                // most keys a token sees
  int whole_norm;                          // queries and keys are normed over all their heads at once instead of per head
  float temp; int temp_every;              // queries are multiplied by 1 + temp ln(floor((pos + 1) / temp_every) + 1) (temp_every 0: not)
  // Sigmoid weights instead of a soft-max: the weight of a key `far` positions back is sigmoid(score - r1 ln(1 + r2 far) + bias), with
  // numbers per head, and nothing is normalised over the keys.
  int sigmoid; const float *r1, *r2, *bias;
  const float* sink;                       // a number per head whose exponential joins the soft-max's normaliser (null: none)
  __host__ __device__ int first_key(int pos) const { return chunked ? pos / window * window : pos >= window ? pos - window + 1 : 0; }
};
struct DeltaDims {
  int heads, kv_heads, dim, vdim, taps; float eps;
  int channel_decay;                       // decay per head and key channel instead of per head
  int sigmoid_gate;                        // output gate sigmoid instead of silu
  int rank_a, rank_g;                      // low-rank projections in front of decay and gate (0: direct)
  __host__ __device__ int channels() const { return 2 * kv_heads * dim + heads * vdim; }
  __host__ __device__ int vdim_p() const { return (vdim + 3) & ~3; }   // row stride of the state
};
// State-space duality: heads of [state][vdim], groups of heads that share B and C; one convolution over x | B | C.
struct SsdDims {
  int heads, vdim, state, groups, taps, norm_groups; float eps;
  __host__ __device__ int inner() const { return heads * vdim; }
  __host__ __device__ int channels() const { return heads * vdim + 2 * groups * state; }
  __host__ __device__ int vdim_p() const { return (vdim + 3) & ~3; }   // row stride of the state
  __host__ __device__ int np() const { return (state + 63) & ~63; }    // strides of the prompt buffers (zero filled)
  __host__ __device__ int xp() const { return (vdim + 15) & ~15; }
};
// Forget-gate linear attention: heads of [dim][vdim], a forget gate per head and channel that also decides what is written.
struct GlaDims {
  int heads, dim, vdim; float eps;
  __host__ __device__ int vdim_p() const { return (vdim + 3) & ~3; }   // row stride of the state
};
// Latent attention: keys (all but a part that turns with the position, one for all heads) and values are products of one latent per
// token, and only the latent and the turned part are cached.
struct LatentDims {
  int heads, dim, rot_dim, vdim, q_rank, kv_rank; float scale, eps;
  int rot; const double* turns; float amp;   // neighbouring pairs of the turned part's first rot dimensions turn by turns[i] full turns a position and grow by amp
  int span;                                  // most keys a token sees
  // a cached row: the latent, then the turned part, each padded to 8 elements with zeros
  __host__ __device__ int lat_c() const { return (kv_rank + 7) & ~7; }
  __host__ __device__ int lat_p() const { return lat_c() + ((rot_dim + 7) & ~7); }
  // a head of the expanded form, padded alike: the key's part from the latent (the query's likewise), the turned part, the value
  __host__ __device__ int dim_e() const { return (dim + 7) & ~7; }
  __host__ __device__ int key_e() const { return dim_e() + ((rot_dim + 7) & ~7); }
  __host__ __device__ int vdim_e() const { return (vdim + 7) & ~7; }
  __host__ __device__ int head_e() const { return dim_e() + vdim_e(); }   // rows of a head in the matrix over the latent
};
constexpr int ATTN_EVERY_KEY = 1 << 30;     // a window that holds every earlier key
struct KvView {                            // what a kernel needs to reach one attention run's pages
  void* base; int64_t page_elems;          // K [kv_head][PAGE_TOKENS][dim_p] then V [kv_head][PAGE_TOKENS][vdim_p]
  const int32_t* table; int ring;          // [slot][ring]
  int64_t v_off;                           // elements from a page's K to its V
};
struct SeqPool {
  int n_seq = 0, n_pages = 0, act_t = ACT_T_BF16, keep = 0;   // keep: the widest window or block (0: no attention run)
  struct AttnRun { AttnDims d; void* base = nullptr; int64_t page_elems = 0, v_off = 0; };
  struct StateRun { int64_t s_elems = 0, h_elems = 0; float* S = nullptr; float* hist = nullptr; };   // state and convolution inputs of one sequence
  std::vector<AttnRun> attn; std::vector<StateRun> state;
  std::vector<AttnDims> readers;                           // the masks of all attention runs, those that read another run's pages too
  int32_t* d_table = nullptr; std::vector<int32_t> table; bool table_dirty = false;
  std::vector<int> free_pages;
  struct Seq { int len = 0; int first_page = 0, end_page = 0; };   // live pages [first_page, end_page)
  std::vector<Seq> seq;

  int alloc(int n_seq, int max_tokens, int act_t);        // after attn / state list their runs
  void release_all();
  int reserve(int s, int new_len);                        // pages for positions [.., new_len)
  void trim(int s);                                       // hands back the pages no window reaches any more
  void free_seq(int s);
  int upload_table();
  int room(int s) const;                                  // tokens sequence s can still take before the pool is out of pages
  int fork(int src, int dst);
  KvView view(int run) const;
};

// ---- grouped attention over pages, in a sliding window or in fixed blocks (cai_attn_paged.hip) ----
// rows of proj: q at column oq ([heads][dim]), k at ok, v at ov.  ok < 0: the pages hold these tokens' keys and values already (an
// earlier run's).  Queries and keys are RMS-normed before the rotation and the score, per head over dim with a shared gain or, with
// whole_norm, over all heads with gains [heads][dim] and [kv_heads][dim] (gain null: not).  og >= 0: the heads' outputs are multiplied
// by the sigmoid of the columns from og on ([heads][vdim]).
struct AttnIn { const float* proj; int64_t ldp; int oq, ok, ov, og; const float *qn, *kn; };
int attn_paged_prep(const AttnDims& d, const KvView& kv, int act_t, const AttnIn& in, const StepRows& r, void* qbuf);     // norms + append; qbuf [row][heads][dim_p]
int attn_paged_rows(const AttnDims& d, const KvView& kv, int act_t, const void* qbuf, const StepRows& r, void* out, int64_t ldo, float* part, size_t part_floats, bool single, const AttnIn& in);
size_t attn_paged_part_floats(const AttnDims& d, int n_rows);   // what n_rows at the longest reach want (many rows share less, in turns)
bool attn_paged_prompt_ok(const AttnDims& d, int act_t);
int attn_paged_prompt(const AttnDims& d, const KvView& kv, const AttnIn& in, const void* qbuf, const StepRows& r, const int32_t* tiles, int n_tiles, void* out, int64_t ldo);
// The same over keys and values laid out in rows, one per position: key columns below `split` and the value at v_off of a head's
// columns, the other key columns shared by all heads in the pages (at `shared` of a page's row).  row0: first row of every entry.
struct FlatKv { const void* base = nullptr; int64_t ld = 0; int head = 0, split = 0, v_off = 0, page_row = 0, shared = 0; const int32_t* row0 = nullptr; };
int attn_flat_prompt(const AttnDims& d, const KvView& kv, const FlatKv& f, const AttnIn& in, const void* qbuf, const StepRows& r, const int32_t* tiles, int n_tiles, void* out, int64_t ldo);
constexpr int ATTN_PROMPT_MIN = 16;        // portions from here on make a step take the prompt kernel
constexpr int ATTN_TILE = 64;              // query rows of one entry per work-group of the prompt kernel

// ---- latent attention (cai_latent.hip) ----
// Columns of proj: the queries' latent, the keys' and values' latent followed by the part that turns, the gate's logits.
// qraw: the queries [row][heads][dim + rot_dim].  up: per head dim_e rows of the key matrix, then vdim_e of the value matrix (over kv_rank).
struct LatentIn { const float* proj; int64_t ldp; int oq, okv, og; const float *qn, *kvn; const float* qraw; int64_t ldq; };
constexpr int LATENT_EXPAND_MIN = 32;      // portions from here on make keys and values of all their positions (expanded form)
// normed latent and turned part into the pages; qlat (null: not): the queries' latent, normed, as rows for their matrix
int latent_append(const LatentDims& d, const KvView& kv, int act_t, const LatentIn& in, const StepRows& r, void* qlat, int64_t ldl);
// The row form: queries are taken into the latent's space (rows of lat_p floats in qabs), meet the cached rows, and their sums of
// latents go through the value matrix.  rows: the rows of the step that take it (null: all); append: the latents join the pages on the way.
int latent_rows(const LatentDims& d, const KvView& kv, int act_t, const LatentIn& in, const cai_qw_s* up, const StepRows& r, const int32_t* rows, int n_rows, bool append, float* qabs,
                float* part, size_t part_floats, void* out, int64_t ldo);
size_t latent_part_floats(const LatentDims& d, int n_rows);
bool latent_expand_ok(const LatentDims& d, int act_t);
// The expanded form's operands: turned queries [row][heads][key_e], and the latents of whole pages as rows of ldc columns.
int latent_queries(const LatentDims& d, const LatentIn& in, const StepRows& r, void* qbuf);
int latent_gather(const LatentDims& d, const KvView& kv, const int32_t* pages, int n_pages, void* rows, int64_t ldc);   // pages: [.][2] slot, page of the sequence

// ---- forget-gate linear attention (cai_gla.hip) ----
// Columns of proj: q (before its silu), the forget gate's logits, v.
struct GlaIn { const float* proj; int64_t ldp; int oq, of, ov; };
struct GlaW { const float *bias, *lower, *norm; };   // of the forget gate [heads * dim] each; [vdim]

// ---- gated delta rule (cai_delta.hip) ----
// Columns of proj: q, k, v (before the convolution), b (write strength), a (decay logits, or their low-rank input), g likewise.
struct DeltaIn { const float* proj; int64_t ldp; int oq, ok, ov, ob, oa, og; };
struct DeltaW {
  const float *cq, *ck, *cv;               // convolution taps [channels][taps]
  const float *rate;                       // -exp(A_log) per head
  const float *dt_bias, *norm;             // [heads] or [heads * dim]; [vdim]
  const cai_qw_s *a2, *g2;                 // low-rank seconds (CAI_BF16), null when direct
};
struct DeltaBuf {                          // per-row scratch of a prompt pass
  float *q, *k, *v, *g, *beta, *o, *za, *zg;
  float *w, *qt, *qk, *gt;                 // chunked form: T [P k], P q, q D k, and the products of decays
};
constexpr int DELTA_CHUNK = 16;            // tokens per chunk
constexpr int DELTA_CHUNK_MIN = 32;        // portions from here on make a step take the chunked form
int delta_prep(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b);
int delta_scan(const DeltaDims& d, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b);
int delta_chunked(const DeltaDims& d, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b, const int32_t* chunks, int n_chunks, const int32_t* chunk0);   // chunks: entry, first row in it; chunk0: first chunk of each entry
int delta_finish(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b, int act_t, void* out, int64_t ldo);
int delta_single(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::StateRun& st, const StepRows& r, int act_t, void* out, int64_t ldo);

int gla_chunked(const GlaDims& d, const GlaIn& in, const GlaW& w, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b, const int32_t* chunks, int n_chunks, const int32_t* chunk0, int act_t, void* out, int64_t ldo);   // uses qt, qk, g, gt, o
int gla_single(const GlaDims& d, const GlaIn& in, const GlaW& w, const SeqPool::StateRun& st, const StepRows& r, int act_t, void* out, int64_t ldo);

// ---- RMS norms around sublayers, depth averages, input convolutions (cai_stream.hip) ----
// A causal convolution over time of a mixer's input h, each channel by itself, added to it.  A sequence's last inputs are kept in a ring of
// `taps` rows (entry position mod taps), one more than a token looks back.
struct InputConv { int taps = 0; const float* w = nullptr; };             // w [taps][width], the last row weighs the current token
struct StreamStep {
  float* x = nullptr; int width = 0; float eps = 0.0f;
  const cai_qw_s* embed = nullptr; float embed_scale = 1.0f;              // x = the token's row times a scale (null: x as it is)
  const float* y = nullptr; int parts = 1; const float* post = nullptr;   // then x += norm(y) post; y is the sum of `parts` rows (null: nothing)
  float* kept = nullptr; int64_t kept_stride = 0; const float* avg = nullptr; int n_kept = 0;   // then kept[n_kept] = x, x = sum of avg[j] kept[j] (avg null: kept only; kept null: neither)
  const float* next = nullptr; void* h = nullptr; int64_t ldh = 0;        // then h = norm(x) next (null: nothing)
  // a convolution behind that norm: single rows take it here (and leave their own input in the ring); others leave the root's
  // reciprocal in `inv`, and launch_input_conv makes h
  InputConv conv; float* ring = nullptr; int64_t ring_elems = 0; float* inv = nullptr;
  // before anything else: the last rows of each entry leave their input - x times inv times keep_gain - in this ring
  float* keep_ring = nullptr; int64_t keep_elems = 0; const float* keep_gain = nullptr; int keep_taps = 0;
};
int launch_stream(const StreamStep& s, int act_t, const StepRows& r, bool single);
int launch_input_conv(const StreamStep& s, int act_t, const StepRows& r);

// ---- state-space duality (cai_ssd.hip) ----
// Columns of proj: z, x | B | C (before the convolution), dt.
struct SsdIn { const float* proj; int64_t ldp; int oz, ox, odt; };
struct SsdW { const float *conv, *conv_b, *dt_bias, *rate, *D, *norm; };   // taps [channels][taps]; rate = -exp(A_log)
struct SsdBuf { float *x, *B, *C, *dt, *cb, *bt, *fac, *y; };               // per-row scratch; per chunk: C B^T and B^T of every group, decay factors of every head
constexpr int SSD_CHUNK = 64, SSD_FACTORS = 4 * SSD_CHUNK + 4;
int ssd_prep(const SsdDims& d, const SsdIn& in, const SsdW& w, const SeqPool::StateRun& st, const StepRows& r, const SsdBuf& b);
int ssd_walk(const SsdDims& d, const SsdW& w, const SeqPool::StateRun& st, const StepRows& r, const SsdBuf& b, const int32_t* chunks, int n_chunks, const int32_t* chunk0);
int ssd_single(const SsdDims& d, const SsdIn& in, const SsdW& w, const SeqPool::StateRun& st, const StepRows& r, const SsdBuf& b);
int ssd_finish(const SsdDims& d, const SsdIn& in, const SsdW& w, const SeqPool::StateRun& st, const StepRows& r, const SsdBuf& b, bool single, int act_t, void* out, int64_t ldo);

// ---- mixtures of experts over bfloat16 weights (cai_experts.hip) ----
// Soft-max scores over all experts; the `top` largest of score + correction are chosen; their weights are the scores over their sum,
// times scale.  ROUTE_AMONG: the `top` largest logits are chosen, and the soft-max is over these alone (times scale).  ROUTE_SIGMOID:
// scores are sigmoids of the logits; of `groups` equal groups of neighbours only the `keep` whose two largest score + correction add up
// to most take part; the weights are the chosen scores as they are (times scale).  A shared expert may run for every token beside them.
enum { ROUTE_ALL = 0, ROUTE_AMONG = 1, ROUTE_SIGMOID = 2 };
struct NetExperts {
  int route = ROUTE_ALL, groups = 1, keep = 1;
  bool gated = true;                       // false: an expert is down(act(up h)), `gateup` holds the up matrices
  int act = CAI_ACT_NONE;                  // of experts that are not gated
  int n = 0, top = 0, ff = 0, ff_shared = 0, glu = GLU_CLAMPED, glu_shared = GLU_CLAMPED;   // ff_shared 0: no shared expert
  float scale = 1.0f, limit = 0.0f, limit_shared = 0.0f;
  cai_qw_s *router = nullptr;              // null: the logits are made elsewhere
  cai_qw_s *gateup = nullptr, *down = nullptr, *s_gateup = nullptr, *s_down = nullptr;   // gateup, down: banks
  const float* correction = nullptr;       // [n], may be null
  int gu_rows() const { return pad_to(ff, 16) * (gated ? 2 : 1); }
  int mid_p() const { return pad_to(ff, LIN_PAD); }
  int shared_p() const { return ff_shared ? pad_to(ff_shared, LIN_PAD) : 0; }
  int active() const { return top * mid_p() + shared_p(); }            // a row's gated activations, one slot after the other
  int max_tiles(int rows, int tile) const { return (rows * top + tile - 1) / tile + n; }
};
constexpr int EXPERTS_MAX = 512, EXPERTS_TOP = 64, EXPERTS_GROUPS = 64;
constexpr int EXPERTS_FEW = 8;             // up to so many rows take the gathering kernels
constexpr int EXPERTS_FEW_WORDS = 2 + EXPERTS_FEW / 2;   // words of a listed expert: itself, its rows, which rows, which of their choices
struct ExpertBuf {
  float *z, *wgt, *y, *ys; int32_t *sel, *order, *tiles, *n_tiles, *few; void *mid, *mid_s;
};
// z: the rows' logits, ldz apart (null: made here); res: the residual update, or, STORE with y null, the outputs of every choice stay in
// b.y [row][experts_parts][width].  beside: a product with the same outputs that joins the
// stream with them, for up to EXPERTS_FEW rows and no shared expert (null: none).
struct BesideLin { const cai_qw_s* w; const void* x; int64_t ldx; LinEpi e; };
inline int experts_parts(const NetExperts& x, int n_rows) { return n_rows == 1 ? 1 : x.top; }
int experts_run(const NetExperts& x, int width, int act_t, const void* h, int64_t ldh, int n_rows, const float* z, int64_t ldz, const ExpertBuf& b, const LinEpi& res, const BesideLin* beside);

// ------------------------------------------------------------------------------------------
// The layered decoder (cai_layered.hip): layers of different kinds, some run several times.
// ------------------------------------------------------------------------------------------
struct NetDelta { DeltaDims d{}; DeltaW w{}; int oq = 0, ok = 0, ov = 0, ob = 0, oa = 0, og = 0; cai_qw_s* out = nullptr; };
struct NetAttn { AttnDims d{}; const float *qn = nullptr, *kn = nullptr, *out_b = nullptr; int oq = 0, ok = 0, ov = 0, og = -1; cai_qw_s* out = nullptr; };
struct NetSsd { SsdDims d{}; SsdW w{}; int oz = 0, ox = 0, odt = 0; cai_qw_s* out = nullptr; };
struct NetLatent { LatentDims d{}; const float *qn = nullptr, *kvn = nullptr; int oq = 0, okv = 0, og = 0; cai_qw_s *uq = nullptr, *up = nullptr, *out = nullptr; };
struct NetGla { GlaDims d{}; GlaW w{}; int oq = 0, of = 0, ov = 0; cai_qw_s* out = nullptr; };
enum { MIX_DELTA = 0, MIX_PARALLEL = 1, MIX_ATTN = 2, MIX_SSD = 3, MIX_LATENT = 4, MIX_GLA = 5 };   // PARALLEL: attention and a delta rule side by side
struct NetLayer {
  int kind = MIX_DELTA;
  cai_qw_s* in = nullptr;                  // every projection of the layer's input, stacked
  const float* in_b = nullptr;             // its bias (null: none)
  NetDelta delta; NetAttn attn; NetSsd ssd; NetLatent latent; NetGla gla;   // (of LATENT, attn.d says what its pages hold)
  const float *gain_left = nullptr, *gain_right = nullptr;   // PARALLEL: gains of the two outputs' RMS norms
  Dyt norm1, norm1b, norm2, norm2b;
  cai_qw_s *gateup = nullptr, *down = nullptr; int ff = 0, glu = GLU_RELU;   // gateup null: no dense feed-forward
  NetExperts experts;                      // n > 0: the feed-forward is a mixture
  // Beside: the feed-forward works beside the mixer on the same stream, each behind an RMS norm of its own, and both results join the
  // stream times a scale per element and the sigmoid of a matrix over the sublayer's input.
  bool beside = false;
  const float *rms1 = nullptr, *rms2 = nullptr, *scale1 = nullptr, *scale2 = nullptr;
  // (`in` begins with the matrix of the mixer's gate logits)  every matrix over the feed-forward's input: its gate logits, then up
  // (squared ReLU; ff rows) or the router
  cai_qw_s* in2 = nullptr; const float* in2_b = nullptr;
  int kv_from = -1;                        // attention over an earlier layer's keys and values
  // Sandwich: x += rms1b(mixer(conv(rms1(x)))), x += rms2b(ff(rms2(x))), RMS norms all, and what goes on is a weighted sum of the results
  // of all layers so far and the embedding output (depth null: the result itself).
  bool sandwich = false;
  const float *rms1b = nullptr, *rms2b = nullptr, *depth = nullptr; InputConv conv;
  bool has_delta() const { return kind == MIX_DELTA || kind == MIX_PARALLEL; }
  bool has_attn() const { return kind == MIX_ATTN || kind == MIX_PARALLEL; }
  bool has_pages() const { return has_attn() || kind == MIX_LATENT; }
  bool has_state() const { return has_delta() || kind == MIX_SSD || kind == MIX_GLA; }
  bool has_mlp() const { return gateup || in2 || experts.n > 0; }
};
// again: the embedding output is added before this run; enter: the stream is replaced by loop_in [stream; embedding output] before it
struct NetRun { int layer; bool again, enter; int attn_run, state_run, conv_run; };
struct LayeredNet;
struct NetSpec {                           // filled by a loader
  int width = 0, vocab = 0; float eps = 0.0f;
  cai_qw_s *embed = nullptr, *head = nullptr;
  cai_qw_s* loop_in = nullptr;             // in front of every pass of the repeated stretch (null: the embedding output is added from the second pass on)
  Dyt final_norm;
  const float* rms_final = nullptr;        // gain of an RMS norm in its place (layers beside, sandwiches)
  float logit_scale = 1.0f, logit_cap = 0.0f;   // logit_cap: logits end as cap tanh(logit / cap) (0: not)
  float embed_scale = 1.0f;                // (sandwiches)
  std::vector<NetLayer> layers;
  int loop_start = 0, loop_stop = 0, loop_times = 1;
  std::vector<cai_qw_s*> weights;          // owned
  std::vector<void*> vectors;              // owned device memory
};
void net_spec_free(NetSpec& s);
int  net_create(NetSpec&& s, int max_tokens, int max_seq, int act_t, LayeredNet** out);
void net_destroy(LayeredNet* n);
// One engine step over any entries.  want[i] != 0: logits of row i are produced, in row order; *_host may be null.
int  net_step(LayeredNet* n, int n_ent, const int32_t* seq, const int32_t* count, const int32_t* tokens, const uint8_t* want,
              float* logits_host, int32_t* argmax_host);
int  net_generate(LayeredNet* n, int seq, int32_t first, int n_tokens, int32_t* out_host);
int  net_len(const LayeredNet* n, int seq);
int  net_room(const LayeredNet* n, int seq);
int  net_pool_pages(const LayeredNet* n);
int  net_peak_pages(const LayeredNet* n, int64_t total, int portion);   // most pages a sequence of `total` tokens fed in such portions holds at once
int  net_rows(const LayeredNet* n, int seq);
int  net_n_runs(const LayeredNet* n);
int  net_reset(LayeredNet* n, int seq);
int  net_fork(LayeredNet* n, int src, int dst);
float* net_logits(LayeredNet* n, int row);         // device row of the last step (null: no such row)
int  net_hidden(LayeredNet* n, int row, float* host);
const NetSpec& net_spec(const LayeredNet* n);
int64_t net_weight_bytes(const LayeredNet* n);
struct NetSnap;
int  net_snapshot(LayeredNet* n, int seq, NetSnap** out);
int  net_restore(LayeredNet* n, int seq, const NetSnap* s);
void net_snap_free(NetSnap* s);

// a decoder around a net (cai_decoder.hip), and the model registry's entry (cai_models.hip)
int decoder_from_net(LayeredNet* n, int max_tokens, int max_seq, cai_decoder_s** out);
// what the scheduler asks of a decoder
int  decoder_pool_pages(cai_decoder_s* d);          // pages all sequences share (0: every sequence has rows of its own)
int  decoder_peak_pages(cai_decoder_s* d, int64_t total, int portion);
bool decoder_bounded(cai_decoder_s* d);             // a sequence ends at max_ctx
bool decoder_keeps_rows(cai_decoder_s* d);          // every wanted row of a batch step stays addressable

}  // namespace cai
