// The layered decoder: decoders whose layers differ in kind and size, where a stretch of layers may run several times with the
// same weights and a cache or state of its own per pass.  Holds the paged pool and state slots (SeqPool), the plan of layer runs,
// and the step function.  A step is any mixture of prompt portions and single tokens of different sequences; a step of single
// tokens only is captured once per width as a graph and replayed.
//
// The residual stream is float.  Behind Dynamic Tanh a sublayer's epilogue adds its result and already leaves the next sublayer's
// normed input, so between two mixers with a dense feed-forward there are three products and nothing else.  Layers whose feed-forward
// works beside the mixer have RMS norms: a small step takes both norms into the one launch of the layer's input matrices and joins
// both results in one other launch; a prompt norms the rows first.  Sublayers that stand in RMS norms (a sandwich) leave their result in
// 32-bit, and one launch a row does everything between it and the next sublayer's input (cai_stream.hip).
#include "cai_layered.hpp"

#include <algorithm>
#include <map>
#include <string.h>

namespace cai {

// ------------------------------------------------------------------------------------------
// pool
// ------------------------------------------------------------------------------------------
int SeqPool::alloc(int n_seq_, int max_tokens, int act_t_)
{
  n_seq = n_seq_; act_t = act_t_;
  keep = 0;
  for (auto& d : readers) keep = std::max(keep, d.window);
  n_pages = attn.empty() ? 0 : (max_tokens + PAGE_TOKENS - 1) / PAGE_TOKENS;
  seq.assign(n_seq, Seq());
  const size_t es = act_t == ACT_T_BF16 ? 2 : 4;
  auto s = ctx().stream;
  for (auto& a : attn) {
    a.v_off = (int64_t)a.d.kv_heads * PAGE_TOKENS * a.d.dim_p;
    a.page_elems = a.v_off + (int64_t)a.d.kv_heads * PAGE_TOKENS * a.d.vdim_p;
    CAI_HIP(hipMalloc(&a.base, (size_t)n_pages * a.page_elems * es));
    CAI_HIP(hipMemsetAsync(a.base, 0, (size_t)n_pages * a.page_elems * es, s));
  }
  for (auto& d : state) {
    for (auto& part : {std::make_pair(&d.S, d.s_elems), std::make_pair(&d.hist, d.h_elems)}) {
      if (!part.second) continue;
      CAI_HIP(hipMalloc((void**)part.first, (size_t)n_seq * part.second * 4));
      CAI_HIP(hipMemsetAsync(*part.first, 0, (size_t)n_seq * part.second * 4, s));
    }
  }
  if (n_pages) {
    table.assign((size_t)n_seq * n_pages, 0);
    CAI_HIP(hipMalloc((void**)&d_table, table.size() * sizeof(int32_t)));
    table_dirty = true;
    for (int p = n_pages - 1; p >= 0; p--) free_pages.push_back(p);
  }
  CAI_HIP(hipStreamSynchronize(s));
  return CAI_OK;
}

void SeqPool::release_all()
{
  for (auto& a : attn) { if (a.base) (void)hipFree(a.base); a.base = nullptr; }
  for (auto& d : state) { if (d.S) (void)hipFree(d.S); if (d.hist) (void)hipFree(d.hist); d.S = d.hist = nullptr; }
  if (d_table) (void)hipFree(d_table);
  d_table = nullptr;
}

int SeqPool::reserve(int s, int new_len)
{
  if (!n_pages) return CAI_OK;
  Seq& q = seq[s];
  const int end = (new_len + PAGE_TOKENS - 1) / PAGE_TOKENS, need = end - q.end_page;
  if (need <= 0) return CAI_OK;
  if (need > (int)free_pages.size())
    return set_error(CAI_ERR_STATE, "cache pool: sequence %d needs %d more pages of %d tokens, %zu of %d are free", s, need, PAGE_TOKENS, free_pages.size(), n_pages);
  for (; q.end_page < end; q.end_page++) {
    table[(size_t)s * n_pages + q.end_page % n_pages] = free_pages.back();
    free_pages.pop_back();
  }
  table_dirty = true;
  return CAI_OK;
}

void SeqPool::trim(int s)
{
  if (!n_pages) return;
  Seq& q = seq[s];
  int oldest = q.len;                                                 // the oldest key the next token sees
  for (auto& d : readers) oldest = std::min(oldest, d.first_key(q.len));
  const int first = oldest / PAGE_TOKENS;
  for (; q.first_page < std::min(first, q.end_page); q.first_page++) free_pages.push_back(table[(size_t)s * n_pages + q.first_page % n_pages]);
}

void SeqPool::free_seq(int s)
{
  Seq& q = seq[s];
  if (n_pages) for (int p = q.first_page; p < q.end_page; p++) free_pages.push_back(table[(size_t)s * n_pages + p % n_pages]);
  q = Seq();
}

int SeqPool::room(int s) const
{
  if (!n_pages) return 1 << 30;
  return (seq[s].end_page + (int)free_pages.size()) * PAGE_TOKENS - seq[s].len;
}

int SeqPool::upload_table()
{
  if (!table_dirty || !n_pages) return CAI_OK;
  CAI_HIP(hipMemcpyAsync(d_table, table.data(), table.size() * sizeof(int32_t), hipMemcpyHostToDevice, ctx().stream));
  CAI_HIP(hipStreamSynchronize(ctx().stream));       // (the host copy changes with the next reservation)
  table_dirty = false;
  return CAI_OK;
}

int SeqPool::fork(int src, int dst)
{
  free_seq(dst);
  const Seq& a = seq[src];
  Seq& b = seq[dst];
  auto s = ctx().stream;
  const size_t es = act_t == ACT_T_BF16 ? 2 : 4;
  if (n_pages) {
    if (a.end_page - a.first_page > (int)free_pages.size())
      return set_error(CAI_ERR_STATE, "cache pool: a copy of sequence %d needs %d pages, %zu are free", src, a.end_page - a.first_page, free_pages.size());
    b.first_page = b.end_page = a.first_page;
    for (; b.end_page < a.end_page; b.end_page++) {
      const int from = table[(size_t)src * n_pages + b.end_page % n_pages], to = free_pages.back();
      free_pages.pop_back();
      table[(size_t)dst * n_pages + b.end_page % n_pages] = to;
      for (auto& r : attn)
        CAI_HIP(hipMemcpyAsync((char*)r.base + (size_t)to * r.page_elems * es, (char*)r.base + (size_t)from * r.page_elems * es, (size_t)r.page_elems * es, hipMemcpyDeviceToDevice, s));
    }
    table_dirty = true;
  }
  for (auto& r : state) {
    if (r.s_elems) CAI_HIP(hipMemcpyAsync(r.S + dst * r.s_elems, r.S + src * r.s_elems, (size_t)r.s_elems * 4, hipMemcpyDeviceToDevice, s));
    if (r.h_elems) CAI_HIP(hipMemcpyAsync(r.hist + dst * r.h_elems, r.hist + src * r.h_elems, (size_t)r.h_elems * 4, hipMemcpyDeviceToDevice, s));
  }
  b.len = a.len;
  return CAI_OK;
}

KvView SeqPool::view(int run) const
{
  const AttnRun& a = attn[run];
  return KvView{a.base, a.page_elems, d_table, n_pages, a.v_off};
}

// ------------------------------------------------------------------------------------------
// small kernels of the step
// ------------------------------------------------------------------------------------------
template <typename AT>
__global__ __launch_bounds__(256) void net_embed_kernel(const uint16_t* e, const int ld, const int32_t* tok, const int width, float* x, float* x0, AT* h, const int64_t ldh, const Dyt next, AT* cat, const int64_t ldc)
{
  const int64_t t = blockIdx.y;
  const uint16_t* row = e + (int64_t)tok[t] * ld;
  for (int i = blockIdx.x * 256 + threadIdx.x; i < width; i += gridDim.x * 256) {
    const float v = __builtin_bit_cast(float, (uint32_t)row[i] << 16);
    x[t * width + i] = v;
    if (x0) x0[t * width + i] = v;
    if (h) h[t * ldh + i] = (AT)dyt(next, v, i);
    if (cat) cat[t * ldc + i] = (AT)v;
  }
}

// Two outputs side by side: each RMS-normed over the width with its own gain, half their sum through `post` onto the residual
// stream (+ add0), then the next sublayer's input.
template <typename AT>
__global__ __launch_bounds__(1024) void net_join_kernel(const float* yl, const float* yr, const float* gl, const float* gr, const int width, const float eps,
                                                        float* x, const float* add0, const Dyt post, const Dyt next, AT* h, const int64_t ldh)
{
  __shared__ float sl[16], sr[16];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x;
  const float *a = yl + t * width, *b = yr + t * width;
  // up to four values a thread stay in registers; wider rows are read again
  float av[4], bv[4], xv[4], glv[4], grv[4];
  float s = 0.0f, q = 0.0f;
#pragma unroll
  for (int u = 0; u < 4; u++) {
    const int i = min(tid + u * 1024, width - 1);
    av[u] = a[i]; bv[u] = b[i]; xv[u] = x[t * width + i];
  }
#pragma unroll
  for (int u = 0; u < 4; u++) { const int i = min(tid + u * 1024, width - 1); glv[u] = gl[i]; grv[u] = gr[i]; }
#pragma unroll
  for (int u = 0; u < 4; u++) if (tid + u * 1024 < width) { s = fmaf(av[u], av[u], s); q = fmaf(bv[u], bv[u], q); }
  for (int i = tid + 4096; i < width; i += 1024) { s = fmaf(a[i], a[i], s); q = fmaf(b[i], b[i], q); }
  for (int o = 32; o; o >>= 1) { s += __shfl_xor(s, o); q += __shfl_xor(q, o); }
  if ((tid & 63) == 0) { sl[tid >> 6] = s; sr[tid >> 6] = q; }
  __syncthreads();
  s = q = 0.0f;
#pragma unroll
  for (int u = 0; u < 16; u++) { s += sl[u]; q += sr[u]; }
  const float il = 1.0f / sqrtf(s / (float)width + eps), ir = 1.0f / sqrtf(q / (float)width + eps);
  auto put = [&](int i, float va, float vb, float vx, float ga, float gb) {
    float v = vx + dyt(post, 0.5f * (va * il * ga + vb * ir * gb), i);
    if (add0) v += add0[t * width + i];
    x[t * width + i] = v;
    h[t * ldh + i] = (AT)dyt(next, v, i);
  };
#pragma unroll
  for (int u = 0; u < 4; u++) if (tid + u * 1024 < width) put(tid + u * 1024, av[u], bv[u], xv[u], glv[u], grv[u]);
  for (int i = tid + 4096; i < width; i += 1024) put(i, a[i], b[i], x[t * width + i], gl[i], gr[i]);
}

// RMS norm of rows of the stream (of those listed in `rows`, or all) with one gain or two; a work-group a row.
template <typename AT>
__global__ __launch_bounds__(256) void net_rms_kernel(const float* x, const int32_t* rows, const int width, const float eps, const float* g1, AT* h1, const float* g2, AT* h2, const int64_t ldh)
{
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const int tid = threadIdx.x;
  const float* v = x + (rows ? rows[t] : t) * width;
  float s = 0.0f;
#pragma unroll 8
  for (int i = tid; i < width; i += 256) s = fmaf(v[i], v[i], s);
  for (int o = 32; o; o >>= 1) s += __shfl_xor(s, o);
  if ((tid & 63) == 0) red[tid >> 6] = s;
  __syncthreads();
  const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)width + eps);
#pragma unroll 4
  for (int i = tid; i < ldh; i += 256) {   // (zeros behind the width)
    const float n = i < width ? v[i] * inv : 0.0f;
    h1[t * ldh + i] = (AT)(i < width ? n * g1[i] : 0.0f);
    if (h2) h2[t * ldh + i] = (AT)(i < width ? n * g2[i] : 0.0f);
  }
}

template <typename AT>
__global__ __launch_bounds__(256) void net_gather_kernel(const AT* h, const int32_t* rows, const int64_t ld, AT* out)
{
  const int64_t src = rows[blockIdx.x];
  for (int64_t i = threadIdx.x; i < ld; i += 256) out[blockIdx.x * ld + i] = h[src * ld + i];
}

// greedy hand-over between two captured steps of one row
__global__ void net_advance_kernel(int32_t* tok, int32_t* pos, const int32_t* best, int32_t* gen, int32_t* gen_idx)
{
  if (threadIdx.x == 0 && blockIdx.x == 0) {
    const int32_t t = best[0]; const int i = gen_idx[0];
    gen[i] = t; gen_idx[0] = i + 1; tok[0] = t; pos[0] += 1;
  }
}

// ------------------------------------------------------------------------------------------
// the net
// ------------------------------------------------------------------------------------------
constexpr int DEC_ROWS = 8;                // widest captured step
constexpr int GEN_STEPS = 8;               // greedy steps per captured launch

struct LayeredNet {
  NetSpec s;
  int act_t = ACT_T_BF16, max_seq = 1;
  size_t es = 2;
  SeqPool pool;
  std::vector<NetRun> runs;
  // widths over all layers
  int wp = 0, ld_proj = 0, ld_mid = 0, ld_att = 0, ld_attl = 0, ld_q = 0, ld_ra = 0, ld_rg = 0;
  int w_q = 0, w_k = 0, w_v = 0, w_g = 0, w_b = 0, w_za = 0, w_zg = 0, w_hd = 0, w_qt = 0, w_qk = 0, w_gt1 = 0;
  int ld_cat = 0, ld_ys = 0, ld_g2 = 0, ld_h2 = 0;
  size_t part_floats = 0;
  int64_t w_cb = 0, w_sx = 0, w_sb = 0, w_sdt = 0, w_sy = 0;                       // state-space scratch, elements per row (cb: per chunk)
  int64_t w_ez = 0, w_ep = 0, w_emid = 0, w_emid_s = 0, w_etiles = 0;              // experts: scores, pairs, activations of a row's pairs, of the shared expert, most tiles of experts
  int ld_ql = 0, ld_qr = 0, ld_lat = 0; int64_t w_qa = 0; bool has_latent = false;   // latent attention: queries' latent, queries, latents, queries in the latent's space
  bool has_parallel = false, has_sandwich = false, looped = false;
  int cap = 0, logit_cap = 0;
  float *x = nullptr, *x0 = nullptr, *proj = nullptr, *yl = nullptr, *yr = nullptr, *part = nullptr, *logits = nullptr;
  void *h = nullptr, *mid = nullptr, *att = nullptr, *attl = nullptr, *qbuf = nullptr, *ra = nullptr, *rgb = nullptr, *hw = nullptr;
  void* cat = nullptr;                     // [stream; embedding] in front of a pass
  void* h2 = nullptr; float* g2 = nullptr; // layers beside: the feed-forward's input, its gate logits and the router's
  float *kept = nullptr, *inv = nullptr;   // sandwiches: embedding output and layer results [layers + 1][rows][width]; reciprocal roots
  void *ql = nullptr; float *qraw = nullptr, *qabs = nullptr;
  int64_t w_flat = 0, flat_cap = 0;        // keys and values of the expanded form, elements per row; rows there are
  void *lat = nullptr, *flat = nullptr;
  DeltaBuf db{};
  SsdBuf sb{};
  ExpertBuf eb{};
  float* am_v = nullptr; int32_t* am_i = nullptr; int32_t* best = nullptr;
  int32_t* d_rows = nullptr; int32_t* h_rows = nullptr; size_t rows_cap = 0;
  int32_t* d_dec = nullptr;                // fixed row arrays of captured steps: tok, pos, slot, first, last [DEC_ROWS each], ent [4 DEC_ROWS], gen_idx
  int32_t* h_dec = nullptr;
  int32_t* d_gen = nullptr; int gen_cap = 0;
  std::map<std::pair<int, int>, hipGraphExec_t> graphs;   // (steps and rows, reach)
  bool use_graph = true;
  std::vector<int> row_of;                 // logits row of the k-th wanted row of the last step
  bool rows_gathered = false;
};

void net_spec_free(NetSpec& s)
{
  for (cai_qw_s* w : s.weights) (void)cai_qw_destroy(w);
  for (void* v : s.vectors) (void)hipFree(v);
  s = NetSpec();
}

static void drop_graphs(LayeredNet* n)
{
  for (auto& g : n->graphs) if (g.second) (void)hipGraphExecDestroy(g.second);
  n->graphs.clear();
}

static void free_rows(LayeredNet* n)
{
  void* p[] = {n->x, n->x0, n->proj, n->yl, n->yr, n->part, n->h, n->mid, n->att, n->attl, n->qbuf, n->ra, n->rgb, n->db.q, n->db.k, n->db.v, n->db.g, n->db.beta, n->db.o, n->db.za, n->db.zg, n->db.w, n->db.qt, n->db.qk, n->db.gt, n->cat, n->h2, n->g2, n->kept, n->inv, n->ql, n->qraw, n->qabs,
               n->sb.x, n->sb.B, n->sb.C, n->sb.dt, n->sb.cb, n->sb.bt, n->sb.fac, n->sb.y, n->eb.z, n->eb.wgt, n->eb.y, n->eb.ys, n->eb.sel, n->eb.order, n->eb.tiles, n->eb.n_tiles, n->eb.few, n->eb.mid, n->eb.mid_s};
  for (void* q : p) if (q) (void)hipFree(q);
  n->x = n->x0 = n->proj = n->yl = n->yr = n->part = nullptr;
  n->h = n->mid = n->att = n->attl = n->qbuf = n->ra = n->rgb = nullptr;
  n->cat = n->h2 = n->ql = nullptr; n->g2 = n->kept = n->inv = n->qraw = n->qabs = nullptr;
  n->db = DeltaBuf{}; n->sb = SsdBuf{}; n->eb = ExpertBuf{};
  n->cap = 0;
}

static int ensure_rows(LayeredNet* n, int rows)
{
  if (n->cap >= rows) return CAI_OK;
  const size_t R = (size_t)std::max(rows, std::max(DEC_ROWS, n->cap + n->cap / 2));
  CAI_HIP(hipStreamSynchronize(ctx().stream));
  drop_graphs(n);
  free_rows(n);
  const int w = n->s.width;
  auto get = [&](void** p, size_t bytes) -> int {
    if (!bytes) return CAI_OK;
    CAI_HIP(hipMalloc(p, bytes));
    CAI_HIP(hipMemsetAsync(*p, 0, bytes, ctx().stream));
    return CAI_OK;
  };
  const size_t RS = R + DELTA_CHUNK + 1;    // the chunked walk requests whole chunks: up to 15 rows (and three values) past the last one
  size_t part = 0;
  // (with bfloat16 activations only steps without a prompt portion take the row form)
  const int part_rows = n->act_t == ACT_T_F32 ? (int)R : std::min((int)R, ATTN_PROMPT_MIN * n->max_seq);
  for (auto& d : n->pool.readers) part = std::max(part, attn_paged_part_floats(d, part_rows));
  for (auto& y : n->s.layers) if (y.kind == MIX_LATENT) part = std::max(part, latent_part_floats(y.latent.d, n->act_t == ACT_T_F32 ? (int)R : std::min((int)R, LATENT_EXPAND_MIN * n->max_seq)));
  n->part_floats = part;
  int rc;
  if ((rc = get((void**)&n->x, R * w * 4)) || (rc = get((void**)&n->x0, n->looped ? R * w * 4 : 0)) || (rc = get((void**)&n->proj, RS * n->ld_proj * 4)) ||
      (rc = get((void**)&n->yl, n->has_parallel || n->has_sandwich ? R * w * 4 : 0)) || (rc = get((void**)&n->yr, n->has_parallel ? R * w * 4 : 0)) || (rc = get((void**)&n->part, part * 4)) ||
      (rc = get(&n->h, R * n->wp * n->es)) || (rc = get(&n->mid, R * n->ld_mid * n->es)) || (rc = get(&n->att, R * n->ld_att * n->es)) ||
      (rc = get(&n->attl, R * n->ld_attl * n->es)) || (rc = get(&n->qbuf, R * n->ld_q * n->es)) || (rc = get(&n->ra, R * n->ld_ra * n->es)) || (rc = get(&n->rgb, R * n->ld_rg * n->es)) ||
      (rc = get((void**)&n->db.q, RS * n->w_q * 4)) || (rc = get((void**)&n->db.k, RS * n->w_k * 4)) || (rc = get((void**)&n->db.v, RS * n->w_v * 4)) ||
      (rc = get((void**)&n->db.g, RS * n->w_g * 4)) || (rc = get((void**)&n->db.beta, RS * n->w_b * 4)) || (rc = get((void**)&n->db.o, RS * n->w_v * 4)) ||
      (rc = get((void**)&n->db.za, R * n->w_za * 4)) || (rc = get((void**)&n->db.zg, R * n->w_zg * 4)) ||
      (rc = get((void**)&n->db.w, RS * n->w_hd * 4)) || (rc = get((void**)&n->db.qt, RS * n->w_qt * 4)) || (rc = get((void**)&n->db.qk, RS * n->w_qk * 4)) ||
      (rc = get((void**)&n->db.gt, std::max(RS * n->w_gt1, (R / DELTA_CHUNK + n->max_seq + 1) * n->w_qt + 4) * 4)) ||
      (rc = get(&n->cat, R * n->ld_cat * n->es)) || (rc = get(&n->h2, R * n->ld_h2 * n->es)) || (rc = get((void**)&n->g2, R * n->ld_g2 * 4)) ||
      (rc = get((void**)&n->kept, n->has_sandwich ? (n->s.layers.size() + 1) * R * w * 4 : 0)) || (rc = get((void**)&n->inv, n->has_sandwich ? R * 4 : 0)) ||
      (rc = get(&n->ql, R * n->ld_ql * n->es)) || (rc = get((void**)&n->qraw, R * n->ld_qr * 4)) || (rc = get((void**)&n->qabs, R * n->w_qa * 4)) ||
      (rc = get((void**)&n->sb.x, (R + SSD_CHUNK) * n->w_sx * 4)) || (rc = get((void**)&n->sb.B, R * n->w_sb * 4)) || (rc = get((void**)&n->sb.C, (R + SSD_CHUNK) * n->w_sb * 4)) ||
      (rc = get((void**)&n->sb.dt, R * n->w_sdt * 4)) || (rc = get((void**)&n->sb.cb, (R / SSD_CHUNK + n->max_seq + 1) * n->w_cb * 4)) || (rc = get((void**)&n->sb.y, R * n->w_sy * 4)) ||
      (rc = get((void**)&n->sb.bt, (R / SSD_CHUNK + n->max_seq + 1) * n->w_sb * SSD_CHUNK * 4)) || (rc = get((void**)&n->sb.fac, (R / SSD_CHUNK + n->max_seq + 1) * n->w_sdt * SSD_FACTORS * 4)) ||
      (rc = get((void**)&n->eb.z, EXPERTS_FEW * n->w_ez * 4)) || (rc = get((void**)&n->eb.few, n->w_ep ? (size_t)EXPERTS_MAX * EXPERTS_FEW_WORDS * 4 : 0)) || (rc = get((void**)&n->eb.sel, R * n->w_ep * 4)) || (rc = get((void**)&n->eb.wgt, R * n->w_ep * 4)) ||
      (rc = get((void**)&n->eb.order, R * n->w_ep * 4)) || (rc = get((void**)&n->eb.y, R * n->w_ep * w * 4)) || (rc = get((void**)&n->eb.ys, R * n->ld_ys * 4)) ||
      (rc = get((void**)&n->eb.tiles, n->w_ep ? ((R * n->w_ep + BANK_TILE - 1) / BANK_TILE + n->w_etiles) * 12 : 0)) || (rc = get((void**)&n->eb.n_tiles, n->w_ep ? 4 : 0)) ||
      (rc = get(&n->eb.mid, R * n->w_emid * n->es)) || (rc = get(&n->eb.mid_s, R * n->w_emid_s * n->es))) return rc;
  CAI_HIP(hipStreamSynchronize(ctx().stream));
  n->cap = (int)R;
  return CAI_OK;
}

// rows of whole pages for the expanded form of latent attention (and a page of slack that the last tile may read)
static int ensure_flat(LayeredNet* n, int64_t rows)
{
  if (n->flat_cap >= rows) return CAI_OK;
  CAI_HIP(hipStreamSynchronize(ctx().stream));
  for (void** p : {&n->lat, &n->flat}) { if (*p) (void)hipFree(*p); *p = nullptr; }
  n->flat_cap = 0;
  const int64_t R = rows + rows / 2 + PAGE_TOKENS;
  CAI_HIP(hipMalloc(&n->lat, (size_t)R * n->ld_lat * 2));
  CAI_HIP(hipMalloc(&n->flat, (size_t)R * n->w_flat * 2));
  CAI_HIP(hipMemsetAsync(n->flat, 0, (size_t)R * n->w_flat * 2, ctx().stream));
  n->flat_cap = R - PAGE_TOKENS;
  return CAI_OK;
}

static int ensure_logits(LayeredNet* n, int rows)
{
  if (n->logit_cap >= rows) return CAI_OK;
  const size_t R = (size_t)std::max(rows, DEC_ROWS);
  CAI_HIP(hipStreamSynchronize(ctx().stream));
  drop_graphs(n);
  void* p[] = {n->logits, n->hw, n->am_v, n->am_i, n->best};
  for (void* q : p) if (q) (void)hipFree(q);
  n->logits = nullptr; n->hw = nullptr; n->am_v = nullptr; n->am_i = nullptr; n->best = nullptr; n->logit_cap = 0;
  const int ame = argmax_scratch_entries(n->s.vocab, (int)R);
  CAI_HIP(hipMalloc((void**)&n->logits, R * n->s.vocab * 4));
  CAI_HIP(hipMalloc(&n->hw, R * n->wp * n->es));
  CAI_HIP(hipMalloc((void**)&n->am_v, (size_t)ame * 4));
  CAI_HIP(hipMalloc((void**)&n->am_i, (size_t)ame * 4));
  CAI_HIP(hipMalloc((void**)&n->best, R * 4));
  n->logit_cap = (int)R;
  return CAI_OK;
}

int net_create(NetSpec&& spec, int max_tokens, int max_seq, int act_t, LayeredNet** out)
{
  LayeredNet* n = new LayeredNet();
  n->s = std::move(spec);
  n->act_t = act_t; n->es = act_t == ACT_T_BF16 ? 2 : 4; n->max_seq = max_seq;
  NetSpec& s = n->s;
  const int L = (int)s.layers.size();
  std::vector<int> last_run(L, -1);        // a layer's latest run with pages of its own
  auto add_run = [&](int l, bool first, int pass) {
    NetRun r{l, first && !s.loop_in && pass > 0, first && s.loop_in, -1, -1, -1};
    NetLayer& y = s.layers[l];
    if (y.has_pages()) {
      // (a sequence longer than the pool exists only if every window is shorter than it: a wider window sees the same keys cut down)
      AttnDims& d = y.attn.d;
      d.span = std::min(d.window, (max_tokens + PAGE_TOKENS - 1) / PAGE_TOKENS * PAGE_TOKENS);
      if (!d.chunked) d.window = d.span;
      y.latent.d.span = d.span;
      if (y.kv_from < 0) { r.attn_run = last_run[l] = (int)n->pool.attn.size(); n->pool.attn.push_back({d}); }
      else r.attn_run = last_run[y.kv_from];
      n->pool.readers.push_back(d);
    }
    if (y.conv.w) {
      SeqPool::StateRun st;
      st.h_elems = (int64_t)y.conv.taps * s.width;
      r.conv_run = (int)n->pool.state.size(); n->pool.state.push_back(st);
    }
    if (y.has_state()) {
      const DeltaDims& d = y.delta.d; const SsdDims& m = y.ssd.d; const GlaDims& a = y.gla.d;
      SeqPool::StateRun st;
      if (y.kind == MIX_GLA) st.s_elems = (int64_t)a.heads * a.dim * a.vdim_p();
      else if (y.kind == MIX_SSD) { st.s_elems = (int64_t)m.heads * m.state * m.vdim_p(); st.h_elems = (int64_t)m.taps * m.channels(); }
      else { st.s_elems = (int64_t)d.heads * d.dim * d.vdim_p(); st.h_elems = (int64_t)d.taps * d.channels(); }
      r.state_run = (int)n->pool.state.size(); n->pool.state.push_back(st);
    }
    n->runs.push_back(r);
  };
  for (int l = 0; l < std::min(s.loop_start, L); l++) add_run(l, false, 0);
  for (int p = 0; p < s.loop_times; p++)
    for (int l = s.loop_start; l < s.loop_stop; l++) add_run(l, l == s.loop_start, p);
  for (int l = s.loop_stop; l < L; l++) add_run(l, false, 0);
  n->looped = !s.loop_in && s.loop_times > 1 && s.loop_stop > s.loop_start;
  n->wp = pad_to(s.width, LIN_PAD);
  if (s.loop_in) n->ld_cat = pad_to(2 * s.width, LIN_PAD);
  auto up = [](auto& a, int64_t v) { if (v > a) a = v; };
  for (const NetLayer& y : s.layers) {
    up(n->ld_proj, pad_to((int)y.in->rows, 4));
    if (y.has_delta()) {
      const DeltaDims& d = y.delta.d;
      up(n->ld_att, pad_to(d.heads * d.vdim, LIN_PAD));
      up(n->w_q, d.kv_heads * d.dim); up(n->w_k, d.kv_heads * d.dim); up(n->w_v, d.heads * d.vdim);
      up(n->w_g, d.channel_decay ? d.heads * d.dim : d.heads); up(n->w_b, d.heads + d.kv_heads);
      up(n->w_hd, d.heads * d.dim); up(n->w_qk, d.heads * DELTA_CHUNK);
      if (d.channel_decay) up(n->w_qt, d.heads * d.dim); else up(n->w_gt1, 2 * d.heads);
      if (d.rank_a) { up(n->ld_ra, pad_to(d.rank_a, LIN_PAD)); up(n->w_za, d.channel_decay ? d.heads * d.dim : d.heads); }
      if (d.rank_g) { up(n->ld_rg, pad_to(d.rank_g, LIN_PAD)); up(n->w_zg, d.heads * d.vdim); }
    }
    if (y.down) up(n->ld_mid, pad_to(y.ff, LIN_PAD));
    if (y.in2) { up(n->ld_g2, pad_to(s.width + y.experts.n, 4)); n->ld_h2 = n->wp; }
    if (y.has_attn()) { up(n->ld_attl, pad_to(y.attn.d.heads * y.attn.d.vdim, LIN_PAD)); up(n->ld_q, y.attn.d.heads * y.attn.d.dim_p); }
    if (y.kind == MIX_PARALLEL) n->has_parallel = true;
    if (y.sandwich) n->has_sandwich = true;
    if (y.kind == MIX_LATENT) {
      const LatentDims& d = y.latent.d;
      n->has_latent = true;
      up(n->ld_attl, pad_to(d.heads * d.vdim, LIN_PAD)); up(n->ld_q, d.heads * d.key_e());
      up(n->ld_ql, pad_to(d.q_rank, LIN_PAD)); up(n->ld_qr, pad_to(d.heads * (d.dim + d.rot_dim), 4)); up(n->w_qa, d.heads * d.lat_p());
      up(n->ld_lat, pad_to(d.kv_rank, LIN_PAD)); up(n->w_flat, d.heads * d.head_e());
    }
    if (y.kind == MIX_GLA) {
      const GlaDims& d = y.gla.d;
      up(n->ld_att, pad_to(d.heads * d.vdim, LIN_PAD));
      up(n->w_v, d.heads * d.vdim); up(n->w_g, d.heads * d.dim); up(n->w_qt, d.heads * d.dim); up(n->w_qk, d.heads * DELTA_CHUNK);
    }
    if (y.kind == MIX_SSD) {
      const SsdDims& d = y.ssd.d;
      up(n->ld_att, pad_to(d.inner(), LIN_PAD));
      up(n->w_sx, d.heads * d.xp()); up(n->w_sb, d.groups * d.np()); up(n->w_sdt, d.heads); up(n->w_sy, d.inner()); up(n->w_cb, d.groups * SSD_CHUNK * SSD_CHUNK);
    }
    if (y.experts.n) {
      const NetExperts& x = y.experts;
      up(n->w_ez, x.n); up(n->w_ep, x.top); up(n->w_etiles, x.n); up(n->w_emid, std::max(x.active(), x.top * x.mid_p())); up(n->w_emid_s, x.shared_p());
      if (x.ff_shared || y.beside) up(n->ld_ys, s.width);
    }
  }
  const char* ng = getenv("CAIHIP_NO_GRAPH");
  n->use_graph = !(ng && ng[0] == '1');
  int rc = n->pool.alloc(max_seq, max_tokens, act_t);
  if (!rc) rc = ensure_rows(n, DEC_ROWS);
  if (!rc) rc = ensure_logits(n, DEC_ROWS);
  if (!rc) {
    hipError_t e = hipMalloc((void**)&n->d_dec, (9 * DEC_ROWS + 1) * sizeof(int32_t));
    if (e == hipSuccess) e = hipHostMalloc((void**)&n->h_dec, (9 * DEC_ROWS + 1) * sizeof(int32_t), hipHostMallocDefault);
    if (e != hipSuccess) rc = hip_fail(e, "layered decoder allocation", __FILE__, __LINE__);
  }
  if (rc) { net_destroy(n); return rc; }
  *out = n;
  return CAI_OK;
}

void net_destroy(LayeredNet* n)
{
  if (!n) return;
  if (ctx().ready) (void)hipStreamSynchronize(ctx().stream);
  drop_graphs(n);
  free_rows(n);
  void* p[] = {n->logits, n->hw, n->am_v, n->am_i, n->best, n->d_rows, n->d_dec, n->d_gen, n->lat, n->flat};
  for (void* q : p) if (q) (void)hipFree(q);
  if (n->h_rows) (void)hipHostFree(n->h_rows);
  if (n->h_dec) (void)hipHostFree(n->h_dec);
  n->pool.release_all();
  net_spec_free(n->s);
  delete n;
}

// Work lists of a step with prompt portions (device pointers): tiles of 64 rows and of DELTA_CHUNK rows (entry, first row in it), and
// the first tile of each entry.  tall: some portion is long enough for the prompt attention kernel; chunked: some portion is long enough
// for the chunked delta rule.
static_assert(ATTN_TILE == SSD_CHUNK, "one list of tiles serves the prompt attention and the state-space walk");
// pages, row0, wide, short_rows: of nets with latent attention - the pages of the entries long enough for its expanded form (slot, page),
// the first row of every such entry there, their tiles, and the rows of the other entries.
struct StepLists {
  const int32_t *tiles = nullptr, *tile0 = nullptr; int n_tiles = 0; bool tall = false;
  const int32_t* chunks = nullptr; int n_chunks = 0; const int32_t* chunk0 = nullptr; bool chunked = false;
  const int32_t *pages = nullptr, *row0 = nullptr, *wide = nullptr, *short_rows = nullptr; int n_pages = 0, n_wide = 0, n_short = 0;
};

template <typename AT>
static void rms_rows_t(LayeredNet* n, const int32_t* rows, int n_rows, const float* g1, void* h1, const float* g2, void* h2)
{
  hipLaunchKernelGGL(net_rms_kernel<AT>, dim3(n_rows), dim3(256), 0, ctx().stream, n->x, rows, n->s.width, n->s.eps, g1, (AT*)h1, g2, (AT*)h2, (int64_t)n->wp);
}
static void rms_rows(LayeredNet* n, const int32_t* rows, int n_rows, const float* g1, void* h1, const float* g2 = nullptr, void* h2 = nullptr)
{
  if (n->act_t == ACT_T_BF16) rms_rows_t<bf16_t>(n, rows, n_rows, g1, h1, g2, h2);
  else rms_rows_t<float>(n, rows, n_rows, g1, h1, g2, h2);
}

static int enqueue_attention(LayeredNet* n, const NetRun& run, const NetLayer& y, const StepRows& r, bool single, const StepLists& lists)
{
  const NetAttn& A = y.attn;
  const int at = n->act_t;
  const AttnIn ain{n->proj, n->ld_proj, A.oq, A.ok, A.ov, A.og, A.qn, A.kn};
  const KvView kv = n->pool.view(run.attn_run);
  int rc;
  if (!single && (rc = attn_paged_prep(A.d, kv, at, ain, r, n->qbuf))) return rc;
  if (!single && lists.tall && attn_paged_prompt_ok(A.d, at)) return attn_paged_prompt(A.d, kv, ain, n->qbuf, r, lists.tiles, lists.n_tiles, n->attl, n->ld_attl);
  return attn_paged_rows(A.d, kv, at, n->qbuf, r, n->attl, n->ld_attl, n->part, n->part_floats, single, ain);
}

// A layer whose feed-forward works beside its mixer: x += scale1 gate1 mixer(norm1(x)) + scale2 gate2 ff(norm2(x)).
static int enqueue_beside(LayeredNet* n, const NetRun& run, const NetLayer& y, const StepRows& r, bool single, const StepLists& lists)
{
  const int R = r.n_rows, w = n->s.width, at = n->act_t;
  const bool few = R <= LIN_FEW;
  int rc;
  LinEpi a, b;
  a.y = n->proj; a.ldy = n->ld_proj; a.bias = y.in_b;
  b.y = n->g2; b.ldy = n->ld_g2; b.bias = y.in2_b;
  if (y.down) { b.mode = EPI_SPLIT; b.split = w; b.act = LIN_RELU_SQUARED; b.h = n->mid; b.ldh = n->ld_mid; }
  if (few) {                               // both norms inside one launch of both stacks of matrices
    const RmsLin first{y.in, y.rms1, a}, second{y.in2, y.rms2, b, y.experts.n ? n->h2 : nullptr, n->wp};
    if ((rc = launch_lin_rms(at, n->x, w, w, n->s.eps, R, first, y.in2 ? &second : nullptr))) return rc;
  } else {
    rms_rows(n, nullptr, R, y.rms1, n->h, y.rms2, y.has_mlp() ? n->h2 : nullptr);
    if ((rc = launch_lin(y.in, at, n->h, n->wp, R, a)) || (y.in2 && (rc = launch_lin(y.in2, at, n->h2, n->wp, R, b)))) return rc;
  }
  if ((rc = enqueue_attention(n, run, y, r, single, lists))) return rc;
  LinEpi m, f;
  m.mode = f.mode = EPI_JOIN; m.y = f.y = n->x; m.ldy = f.ldy = w;
  m.mult = y.scale1; m.gate = n->proj; m.ldg = n->ld_proj;
  f.mult = y.scale2; f.gate = n->g2; f.ldg = n->ld_g2;
  const BesideLin o{y.attn.out, n->attl, n->ld_attl, m};
  if (few && y.experts.n) return experts_run(y.experts, w, at, n->h2, n->wp, R, n->g2 + w, n->ld_g2, n->eb, f, &o);
  if (few && y.down) return launch_lin_pair(at, R, y.attn.out, n->attl, n->ld_attl, m, y.down, n->mid, n->ld_mid, f);
  if ((rc = launch_lin(y.attn.out, at, n->attl, n->ld_attl, R, m))) return rc;
  if (y.experts.n) return experts_run(y.experts, w, at, n->h2, n->wp, R, n->g2 + w, n->ld_g2, n->eb, f, nullptr);
  return y.down ? launch_lin(y.down, at, n->mid, n->ld_mid, R, f) : CAI_OK;
}

static int enqueue_latent(LayeredNet* n, const NetRun& run, const NetLayer& y, const StepRows& r, bool single, const StepLists& lists)
{
  const NetLatent& L = y.latent;
  const LatentDims& d = L.d;
  const int at = n->act_t, R = r.n_rows;
  const LatentIn in{n->proj, n->ld_proj, L.oq, L.okv, L.og, L.qn, L.kvn, n->qraw, n->ld_qr};
  const KvView kv = n->pool.view(run.attn_run);
  const bool few = R <= LIN_FEW;
  int rc;
  if (!single && (rc = latent_append(d, kv, at, in, r, few ? nullptr : n->ql, n->ld_ql))) return rc;
  LinEpi e; e.y = n->qraw; e.ldy = n->ld_qr;
  if (few) rc = launch_lin_rms(at, n->proj + L.oq, n->ld_proj, d.q_rank, d.eps, R, RmsLin{L.uq, L.qn, e}, nullptr);
  else rc = launch_lin(L.uq, at, n->ql, n->ld_ql, R, e);
  if (rc) return rc;
  const bool wide = lists.n_wide > 0 && latent_expand_ok(d, at);
  if (!wide || lists.n_short) {
    const int32_t* rows = wide ? lists.short_rows : nullptr;
    if ((rc = latent_rows(d, kv, at, in, L.up, r, rows, wide ? lists.n_short : R, single, n->qabs, n->part, n->part_floats, n->attl, n->ld_attl))) return rc;
  }
  if (!wide) return CAI_OK;
  // the expanded form: keys and values of all positions of the longer entries
  AttnDims a{};
  a.heads = a.kv_heads = d.heads; a.dim = a.dim_p = d.key_e(); a.vdim = d.vdim; a.vdim_p = d.vdim_e(); a.window = y.attn.d.window; a.span = d.span; a.scale = d.scale;
  const int64_t ldf = (int64_t)d.heads * d.head_e(), ldc = L.up->ld;
  const FlatKv f{n->flat, ldf, d.head_e(), d.dim_e(), d.dim_e(), d.lat_p(), d.lat_c(), lists.row0};
  const AttnIn ain{n->proj, n->ld_proj, 0, -1, -1, L.og, nullptr, nullptr};
  LinEpi x; x.mode = EPI_SPLIT; x.split = 0; x.h = n->flat; x.ldh = ldf;
  if ((rc = latent_queries(d, in, r, n->qbuf)) || (rc = latent_gather(d, kv, lists.pages, lists.n_pages, n->lat, ldc)) ||
      (rc = launch_lin(L.up, at, n->lat, ldc, lists.n_pages * PAGE_TOKENS, x))) return rc;
  return attn_flat_prompt(a, kv, f, ain, n->qbuf, r, lists.wide, lists.n_wide, n->attl, n->ld_attl);
}

// Norm (and convolution) in front of run i's mixer, or in front of the logits.
static void sandwich_lead(LayeredNet* n, size_t i, StreamStep& s)
{
  if (i >= n->runs.size()) { s.next = n->s.rms_final; return; }
  const NetLayer& y = n->s.layers[n->runs[i].layer];
  s.next = y.rms1; s.conv = y.conv;
  if (y.conv.w) { const SeqPool::StateRun& c = n->pool.state[n->runs[i].conv_run]; s.ring = c.hist; s.ring_elems = c.h_elems; }
}
static int sandwich_stream(LayeredNet* n, const StreamStep& s, const StepRows& r, bool single)
{
  const int rc = launch_stream(s, n->act_t, r, single);
  return rc || single || !s.conv.w ? rc : launch_input_conv(s, n->act_t, r);
}
static StreamStep sandwich_step(LayeredNet* n)
{
  StreamStep s;
  s.x = n->x; s.width = n->s.width; s.eps = n->s.eps; s.h = n->h; s.ldh = n->wp; s.inv = n->inv;
  return s;
}

// A layer whose sublayers stand in RMS norms; its mixer's input is in h already.
static int enqueue_sandwich(LayeredNet* n, size_t i, const StepRows& r, bool single, const StepLists& lists)
{
  const NetRun& run = n->runs[i];
  const NetLayer& y = n->s.layers[run.layer];
  const int R = r.n_rows, w = n->s.width, at = n->act_t;
  int rc;
  { LinEpi e; e.y = n->proj; e.ldy = n->ld_proj; e.bias = y.in_b; if ((rc = launch_lin(y.in, at, n->h, n->wp, R, e))) return rc; }
  const cai_qw_s* out = y.attn.out; const void* heads = n->attl; int ldo = n->ld_attl;
  if (y.kind == MIX_LATENT) { out = y.latent.out; rc = enqueue_latent(n, run, y, r, single, lists); }
  else if (y.kind == MIX_GLA) {
    const NetGla& G = y.gla;
    const GlaIn gin{n->proj, n->ld_proj, G.oq, G.of, G.ov};
    const SeqPool::StateRun& st = n->pool.state[run.state_run];
    out = G.out; heads = n->att; ldo = n->ld_att;
    rc = single ? gla_single(G.d, gin, G.w, st, r, at, n->att, ldo) : gla_chunked(G.d, gin, G.w, st, r, n->db, lists.chunks, lists.n_chunks, lists.chunk0, at, n->att, ldo);
  } else rc = enqueue_attention(n, run, y, r, single, lists);
  if (rc) return rc;
  { LinEpi e; e.y = n->yl; e.ldy = w; if ((rc = launch_lin(out, at, heads, ldo, R, e))) return rc; }
  StreamStep s = sandwich_step(n);
  s.y = n->yl; s.post = y.rms1b;
  if (y.conv.w && !single) { const SeqPool::StateRun& c = n->pool.state[run.conv_run]; s.keep_ring = c.hist; s.keep_elems = c.h_elems; s.keep_gain = y.rms1; s.keep_taps = y.conv.taps; }
  if (y.has_mlp()) {
    s.next = y.rms2;
    if ((rc = launch_stream(s, at, r, single))) return rc;
    LinEpi apart;
    if ((rc = experts_run(y.experts, w, at, n->h, n->wp, R, nullptr, 0, n->eb, apart, nullptr))) return rc;
    s = sandwich_step(n);
    s.y = n->eb.y; s.parts = experts_parts(y.experts, R); s.post = y.rms2b;
  }
  s.kept = n->kept; s.kept_stride = (int64_t)n->cap * w; s.n_kept = (int)i + 1; s.avg = y.depth;
  sandwich_lead(n, i + 1, s);
  return sandwich_stream(n, s, r, single);
}

// Logits of the wanted rows (null: all), and their greedy choices.  A sandwich's last stream step has normed the rows already.
static int enqueue_logits(LayeredNet* n, const int32_t* want, int n_want)
{
  if (n_want > 0) {
    const NetSpec& s = n->s;
    const int w = s.width, at = n->act_t;
    const bool norm = s.rms_final && !n->has_sandwich;
    auto st = ctx().stream;
    const void* hs = n->h;
    int rc;
    LinEpi e; e.y = n->logits; e.ldy = s.vocab; e.scale = s.logit_scale;
    if (s.logit_cap > 0.0f) { e.act = LIN_SOFT_CAP; e.limit = s.logit_cap; }
    if (norm && !want && n_want <= LIN_FEW) {
      if ((rc = launch_lin_rms(at, n->x, w, w, s.eps, n_want, RmsLin{s.head, s.rms_final, e, n->h, n->wp}, nullptr))) return rc;
      hs = nullptr;
    } else if (norm) {
      if (want) hs = n->hw;
      rms_rows(n, want, n_want, s.rms_final, (void*)hs);
    } else if (want) {
      if (at == ACT_T_BF16) hipLaunchKernelGGL(net_gather_kernel<bf16_t>, dim3(n_want), dim3(256), 0, st, (const bf16_t*)n->h, want, (int64_t)n->wp, (bf16_t*)n->hw);
      else hipLaunchKernelGGL(net_gather_kernel<float>, dim3(n_want), dim3(256), 0, st, (const float*)n->h, want, (int64_t)n->wp, (float*)n->hw);
      hs = n->hw;
    }
    if (hs && (rc = launch_lin(s.head, at, hs, n->wp, n_want, e))) return rc;
    launch_argmax(n->logits, s.vocab, n_want, n->best, n->am_v, n->am_i);
  }
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

// One step over the rows of `r`.  single: every entry is one row (the decode kernels).  want: device list of the rows whose
// logits are produced (null: all rows, in order).
static int enqueue_net(LayeredNet* n, const StepRows& r, bool single, const StepLists& lists, const int32_t* want, int n_want)
{
  const NetSpec& s = n->s;
  const int R = r.n_rows, w = s.width, at = n->act_t;
  auto st = ctx().stream;
  int rc;
  auto norm1_of = [&](size_t i) -> const Dyt& { return s.layers[n->runs[i].layer].norm1; };
  const dim3 eg((unsigned)std::min((w + 255) / 256, 32), R);
  if (n->has_sandwich) {
    StreamStep e = sandwich_step(n);
    e.embed = s.embed; e.embed_scale = s.embed_scale; e.kept = n->kept; e.kept_stride = (int64_t)n->cap * w;
    sandwich_lead(n, 0, e);
    if ((rc = sandwich_stream(n, e, r, single))) return rc;
    for (size_t i = 0; i < n->runs.size(); i++) if ((rc = enqueue_sandwich(n, i, r, single, lists))) return rc;
    return enqueue_logits(n, want, n_want);
  }
  // where the stream goes after the last sublayer before run i: the norm of what follows, or as it is in front of loop_in
  auto lead_to = [&](size_t i, LinEpi& e) {
    if (i < n->runs.size() && n->runs[i].enter) { e.next = Dyt(); e.h = n->cat; e.ldh = n->ld_cat; return; }
    e.next = i < n->runs.size() ? norm1_of(i) : s.final_norm; e.h = n->h; e.ldh = n->wp;
    if (i < n->runs.size() && n->runs[i].again) { e.add0 = n->x0; e.ld0 = w; }
  };
  LinEpi first;
  if (!s.rms_final) lead_to(0, first);
#define EMBED(T) hipLaunchKernelGGL(net_embed_kernel<T>, eg, dim3(256), 0, st, (const uint16_t*)s.embed->data, (int)s.embed->ld, r.tok, w, n->x, n->x0, (T*)first.h, first.ldh, first.next, s.loop_in ? (T*)n->cat + w : nullptr, (int64_t)n->ld_cat)
  if (at == ACT_T_BF16) EMBED(bf16_t); else EMBED(float);
#undef EMBED
  for (size_t i = 0; i < n->runs.size(); i++) {
    const NetRun& run = n->runs[i];
    const NetLayer& y = s.layers[run.layer];
    if (y.beside) {
      if ((rc = enqueue_beside(n, run, y, r, single, lists))) return rc;
      continue;
    }
    if (run.enter) {
      LinEpi e; e.mode = EPI_RESIDUAL; e.fresh = true; e.y = n->x; e.ldy = w; e.h = n->h; e.ldh = n->wp; e.next = y.norm1;
      if ((rc = launch_lin(s.loop_in, at, n->cat, n->ld_cat, R, e))) return rc;
    }
    { LinEpi e; e.y = n->proj; e.ldy = n->ld_proj; e.bias = y.in_b; if ((rc = launch_lin(y.in, at, n->h, n->wp, R, e))) return rc; }
    LinEpi res; res.mode = EPI_RESIDUAL; res.y = n->x; res.ldy = w; res.post = y.norm1b;
    if (y.has_mlp()) { res.next = y.norm2; res.h = n->h; res.ldh = n->wp; }
    else lead_to(i + 1, res);
    if (y.has_delta()) {
      const NetDelta& D = y.delta;
      const DeltaIn din{n->proj, n->ld_proj, D.oq, D.ok, D.ov, D.ob, D.oa, D.og};
      const SeqPool::StateRun& ds = n->pool.state[run.state_run];
      if (single) {
        if ((rc = delta_single(D.d, din, D.w, ds, r, at, n->att, n->ld_att))) return rc;
      } else {
        if (D.d.rank_a) {
          LinEpi e; e.y = n->db.za; e.ldy = D.w.a2->rows;
          if ((rc = launch_pack_rows(n->proj, n->ld_proj, D.oa, D.d.rank_a, R, at, n->ra, n->ld_ra)) || (rc = launch_lin(D.w.a2, at, n->ra, n->ld_ra, R, e))) return rc;
        }
        if (D.d.rank_g) {
          LinEpi e; e.y = n->db.zg; e.ldy = D.w.g2->rows;
          if ((rc = launch_pack_rows(n->proj, n->ld_proj, D.og, D.d.rank_g, R, at, n->rgb, n->ld_rg)) || (rc = launch_lin(D.w.g2, at, n->rgb, n->ld_rg, R, e))) return rc;
        }
        if ((rc = delta_prep(D.d, din, D.w, ds, r, n->db)) ||
            (rc = lists.chunked ? delta_chunked(D.d, ds, r, n->db, lists.chunks, lists.n_chunks, lists.chunk0) : delta_scan(D.d, ds, r, n->db)) ||
            (rc = delta_finish(D.d, din, D.w, ds, r, n->db, at, n->att, n->ld_att))) return rc;
      }
    }
    if (y.kind == MIX_SSD) {
      const NetSsd& M = y.ssd;
      const SsdIn sin{n->proj, n->ld_proj, M.oz, M.ox, M.odt};
      const SeqPool::StateRun& ss = n->pool.state[run.state_run];
      if (single) rc = ssd_single(M.d, sin, M.w, ss, r, n->sb);
      else if (!(rc = ssd_prep(M.d, sin, M.w, ss, r, n->sb))) rc = ssd_walk(M.d, M.w, ss, r, n->sb, lists.tiles, lists.n_tiles, lists.tile0);
      if (rc || (rc = ssd_finish(M.d, sin, M.w, ss, r, n->sb, single, at, n->att, n->ld_att))) return rc;
    }
    if (y.has_attn() && (rc = enqueue_attention(n, run, y, r, single, lists))) return rc;
    if (y.kind == MIX_PARALLEL) {
      LinEpi el, er; el.y = n->yl; er.y = n->yr; el.ldy = er.ldy = w;
      if ((rc = launch_lin(y.attn.out, at, n->attl, n->ld_attl, R, el)) || (rc = launch_lin(y.delta.out, at, n->att, n->ld_att, R, er))) return rc;
#define JOIN(T) hipLaunchKernelGGL(net_join_kernel<T>, dim3(R), dim3(1024), 0, st, n->yl, n->yr, y.gain_left, y.gain_right, w, s.eps, n->x, res.add0, res.post, res.next, (T*)res.h, res.ldh)
      if (at == ACT_T_BF16) JOIN(bf16_t); else JOIN(float);
#undef JOIN
    } else if (y.kind == MIX_ATTN) {
      res.bias = y.attn.out_b;
      if ((rc = launch_lin(y.attn.out, at, n->attl, n->ld_attl, R, res))) return rc;
      res.bias = nullptr;
    } else if ((rc = launch_lin(y.kind == MIX_SSD ? y.ssd.out : y.delta.out, at, n->att, n->ld_att, R, res))) return rc;
    if (!y.has_mlp()) continue;
    res.post = y.norm2b;
    lead_to(i + 1, res);
    if (y.experts.n) {
      if ((rc = experts_run(y.experts, w, at, n->h, n->wp, R, nullptr, 0, n->eb, res, nullptr))) return rc;
      continue;
    }
    LinEpi g; g.mode = EPI_GLU; g.h = n->mid; g.ldh = n->ld_mid; g.glu = y.glu;
    if ((rc = launch_lin(y.gateup, at, n->h, n->wp, R, g)) || (rc = launch_lin(y.down, at, n->mid, n->ld_mid, R, res))) return rc;
  }
  return enqueue_logits(n, want, n_want);
}

static StepRows dec_rows(const LayeredNet* n, int R, int reach)
{
  int32_t* d = n->d_dec;
  return StepRows{d, d + DEC_ROWS, d + 2 * DEC_ROWS, d + 3 * DEC_ROWS, d + 4 * DEC_ROWS, d + 5 * DEC_ROWS, R, R, reach};
}

// `steps` captured steps of R single rows, with the greedy hand-over after each when gen is set (R = 1).  No position reaches `end`:
// launches over the keys are sized by the next power of two (or by the widest window), so that a sequence captures a few times while
// it grows.
static int run_captured(LayeredNet* n, int R, int steps, bool gen, int end)
{
  auto st = ctx().stream;
  int reach = 256;
  while (reach < end && reach < n->pool.keep) reach *= 2;
  if (reach >= n->pool.keep) reach = std::max(n->pool.keep, 1);
  const StepRows r = dec_rows(n, R, reach);
  auto body = [&]() -> int {
    for (int i = 0; i < steps; i++) {
      const int rc = enqueue_net(n, r, true, StepLists(), nullptr, R);
      if (rc) return rc;
      if (gen) hipLaunchKernelGGL(net_advance_kernel, dim3(1), dim3(64), 0, st, n->d_dec, n->d_dec + DEC_ROWS, n->best, n->d_gen, n->d_dec + 9 * DEC_ROWS);
    }
    return CAI_OK;
  };
  if (!n->use_graph) return body();
  hipGraphExec_t& ge = n->graphs[{(gen ? 1000 : 0) + steps * 16 + R, reach}];
  if (!ge) {
    hipGraph_t g = nullptr;
    CAI_HIP(hipStreamBeginCapture(st, hipStreamCaptureModeThreadLocal));
    const int rc = body();
    const hipError_t e = hipStreamEndCapture(st, &g);
    if (rc) { if (g) (void)hipGraphDestroy(g); return rc; }
    if (e != hipSuccess) return hip_fail(e, "hipStreamEndCapture", __FILE__, __LINE__);
    const hipError_t e2 = hipGraphInstantiate(&ge, g, nullptr, nullptr, 0);
    (void)hipGraphDestroy(g);
    if (e2 != hipSuccess) { ge = nullptr; return hip_fail(e2, "hipGraphInstantiate", __FILE__, __LINE__); }
  }
  CAI_HIP(hipGraphLaunch(ge, st));
  return CAI_OK;
}

int net_step(LayeredNet* n, int n_ent, const int32_t* seq, const int32_t* count, const int32_t* tokens, const uint8_t* want, float* logits_host, int32_t* argmax_host)
{
  CAI_REQUIRE(n_ent >= 1 && n_ent <= n->max_seq, "engine step: %d entries for %d sequences", n_ent, n->max_seq);
  int64_t R64 = 0; bool single = true;
  std::vector<uint8_t> seen(n->max_seq, 0);
  for (int e = 0; e < n_ent; e++) {
    CAI_REQUIRE(seq[e] >= 0 && seq[e] < n->max_seq && !seen[seq[e]], "engine step: entry %d names sequence %d (of %d, each once)", e, seq[e], n->max_seq);
    CAI_REQUIRE(count[e] >= 1, "engine step: entry %d has %d tokens", e, count[e]);
    seen[seq[e]] = 1; R64 += count[e]; single = single && count[e] == 1;
  }
  CAI_REQUIRE(R64 <= (1 << 17), "engine step: %lld rows", (long long)R64);
  const int R = (int)R64;
  for (int i = 0; i < R; i++) CAI_REQUIRE(tokens[i] >= 0 && tokens[i] < n->s.vocab, "engine step: token %d outside vocab %d", tokens[i], n->s.vocab);
  // pages for all entries or for none
  if (n->pool.n_pages) {
    int need = 0;
    for (int e = 0; e < n_ent; e++) { const auto& q = n->pool.seq[seq[e]]; need += std::max(0, (q.len + count[e] + PAGE_TOKENS - 1) / PAGE_TOKENS - q.end_page); }
    if (need > (int)n->pool.free_pages.size())
      return set_error(CAI_ERR_STATE, "engine step: %d more cache pages of %d tokens needed, %zu of %d free", need, PAGE_TOKENS, n->pool.free_pages.size(), n->pool.n_pages);
  }
  int rc;
  for (int e = 0; e < n_ent; e++) if ((rc = n->pool.reserve(seq[e], n->pool.seq[seq[e]].len + count[e]))) return rc;
  if ((rc = n->pool.upload_table())) return rc;
  auto st = ctx().stream;
  std::vector<int32_t> wrows;
  for (int i = 0; i < R; i++) if (want && want[i]) wrows.push_back(i);
  const int W = (int)wrows.size();
  n->row_of.clear();
  if (single && R <= DEC_ROWS) {
    int32_t* hd = n->h_dec;
    int end = 0;
    for (int e = 0; e < R; e++) {
      const int pos = n->pool.seq[seq[e]].len;
      end = std::max(end, pos + 1);
      hd[e] = tokens[e]; hd[DEC_ROWS + e] = pos; hd[2 * DEC_ROWS + e] = seq[e]; hd[3 * DEC_ROWS + e] = e; hd[4 * DEC_ROWS + e] = e;
      int32_t* en = hd + 5 * DEC_ROWS + 4 * e; en[0] = seq[e]; en[1] = e; en[2] = 1; en[3] = pos;
    }
    CAI_HIP(hipMemcpyAsync(n->d_dec, hd, 9 * DEC_ROWS * sizeof(int32_t), hipMemcpyHostToDevice, st));
    if ((rc = run_captured(n, R, 1, false, end))) return rc;
    n->row_of = wrows; n->rows_gathered = false;
  } else {
    // rows, entries, tiles of the prompt attention kernel, wanted rows
    std::vector<int32_t> tiles, tile0, chunks, chunk0, pages, row0, wide, short_rows;
    bool tall = false, chunked = false;
    int end = 0;
    for (int e = 0; e < n_ent; e++) {
      end = std::max(end, n->pool.seq[seq[e]].len + count[e]);
      tall = tall || count[e] >= ATTN_PROMPT_MIN; chunked = chunked || count[e] >= DELTA_CHUNK_MIN;
      chunk0.push_back((int)chunks.size() / 2); tile0.push_back((int)tiles.size() / 2);
      for (int t = 0; t < count[e]; t += ATTN_TILE) { tiles.push_back(e); tiles.push_back(t); }
      for (int t = 0; t < count[e]; t += DELTA_CHUNK) { chunks.push_back(e); chunks.push_back(t); }
    }
    for (int e = 0, i = 0; n->has_latent && e < n_ent; i += count[e++]) {
      row0.push_back((int)pages.size() / 2 * PAGE_TOKENS);
      if (count[e] < LATENT_EXPAND_MIN) { for (int t = 0; t < count[e]; t++) short_rows.push_back(i + t); continue; }
      for (int p = 0; p * PAGE_TOKENS < n->pool.seq[seq[e]].len + count[e]; p++) { pages.push_back(seq[e]); pages.push_back(p); }
      for (int t = 0; t < count[e]; t += ATTN_TILE) { wide.push_back(e); wide.push_back(t); }
    }
    std::vector<const std::vector<int32_t>*> parts = {&tiles, &tile0, &chunks, &chunk0, &pages, &row0, &wide, &short_rows, &wrows};
    size_t need = (size_t)5 * R + 4 * n_ent;
    for (auto* v : parts) need += v->size();
    if (n->rows_cap < need) {
      CAI_HIP(hipStreamSynchronize(st));
      if (n->d_rows) (void)hipFree(n->d_rows);
      if (n->h_rows) (void)hipHostFree(n->h_rows);
      n->d_rows = nullptr; n->h_rows = nullptr; n->rows_cap = 0;
      CAI_HIP(hipMalloc((void**)&n->d_rows, need * 2 * sizeof(int32_t)));
      CAI_HIP(hipHostMalloc((void**)&n->h_rows, need * 2 * sizeof(int32_t), hipHostMallocDefault));
      n->rows_cap = need * 2;
    }
    if ((rc = ensure_rows(n, R)) || (rc = ensure_logits(n, std::max(W, 1))) || (pages.size() && n->act_t == ACT_T_BF16 && (rc = ensure_flat(n, (int64_t)pages.size() / 2 * PAGE_TOKENS)))) return rc;
    int32_t* hr = n->h_rows;
    int32_t* ent = hr + 5 * R;
    for (int e = 0, i = 0; e < n_ent; e++) {
      const int pos0 = n->pool.seq[seq[e]].len, r0 = i;
      ent[4 * e] = seq[e]; ent[4 * e + 1] = r0; ent[4 * e + 2] = count[e]; ent[4 * e + 3] = pos0;
      for (int t = 0; t < count[e]; t++, i++) { hr[i] = tokens[i]; hr[R + i] = pos0 + t; hr[2 * R + i] = seq[e]; hr[3 * R + i] = r0; hr[4 * R + i] = r0 + count[e] - 1; }
    }
    int32_t* ht = ent + 4 * n_ent;
    for (auto* v : parts) ht = std::copy(v->begin(), v->end(), ht);
    CAI_HIP(hipMemcpyAsync(n->d_rows, hr, need * sizeof(int32_t), hipMemcpyHostToDevice, st));
    const int32_t* d = n->d_rows;
    const StepRows r{d, d + R, d + 2 * R, d + 3 * R, d + 4 * R, d + 5 * R, R, n_ent, end};
    const int32_t* at = d + 5 * R + 4 * n_ent;
    auto next = [&](const std::vector<int32_t>& v) { const int32_t* p = at; at += v.size(); return p; };
    StepLists lists;
    lists.tiles = next(tiles); lists.n_tiles = (int)tiles.size() / 2; lists.tile0 = next(tile0); lists.tall = tall;
    lists.chunks = next(chunks); lists.n_chunks = (int)chunks.size() / 2; lists.chunk0 = next(chunk0); lists.chunked = chunked;
    lists.pages = next(pages); lists.n_pages = (int)pages.size() / 2; lists.row0 = next(row0);
    lists.wide = next(wide); lists.n_wide = (int)wide.size() / 2; lists.short_rows = next(short_rows); lists.n_short = (int)short_rows.size();
    if ((rc = enqueue_net(n, r, false, lists, next(wrows), W))) return rc;
    for (int k = 0; k < W; k++) n->row_of.push_back(k);
    n->rows_gathered = true;
  }
  for (int k = 0; k < W; k++) {
    // (consecutive logits rows come back in one copy)
    int k2 = k; while (k2 + 1 < W && n->row_of[k2 + 1] == n->row_of[k2] + 1) k2++;
    if (logits_host) CAI_HIP(hipMemcpyAsync(logits_host + (size_t)k * n->s.vocab, n->logits + (size_t)n->row_of[k] * n->s.vocab, (size_t)(k2 - k + 1) * n->s.vocab * 4, hipMemcpyDeviceToHost, st));
    if (argmax_host) CAI_HIP(hipMemcpyAsync(argmax_host + k, n->best + n->row_of[k], (size_t)(k2 - k + 1) * 4, hipMemcpyDeviceToHost, st));
    k = k2;
  }
  CAI_HIP(hipStreamSynchronize(st));
  for (int e = 0; e < n_ent; e++) { n->pool.seq[seq[e]].len += count[e]; n->pool.trim(seq[e]); }
  return CAI_OK;
}

int net_generate(LayeredNet* n, int seq, int32_t first, int n_tokens, int32_t* out_host)
{
  auto st = ctx().stream;
  CAI_REQUIRE(first >= 0 && first < n->s.vocab, "greedy generation: token %d outside vocab %d", first, n->s.vocab);
  if (n->gen_cap < n_tokens) {
    CAI_HIP(hipStreamSynchronize(st));
    if (n->d_gen) (void)hipFree(n->d_gen);
    n->d_gen = nullptr; n->gen_cap = 0;
    drop_graphs(n);
    CAI_HIP(hipMalloc((void**)&n->d_gen, (size_t)std::max(n_tokens, 256) * 4));
    n->gen_cap = std::max(n_tokens, 256);
  }
  SeqPool::Seq& q = n->pool.seq[seq];
  int32_t* hd = n->h_dec;
  hd[0] = first; hd[DEC_ROWS] = q.len; hd[2 * DEC_ROWS] = seq; hd[3 * DEC_ROWS] = 0; hd[4 * DEC_ROWS] = 0;
  hd[5 * DEC_ROWS] = seq; hd[5 * DEC_ROWS + 1] = 0; hd[5 * DEC_ROWS + 2] = 1; hd[5 * DEC_ROWS + 3] = q.len; hd[9 * DEC_ROWS] = 0;
  CAI_HIP(hipMemcpyAsync(n->d_dec, hd, (9 * DEC_ROWS + 1) * sizeof(int32_t), hipMemcpyHostToDevice, st));
  for (int i = 0; i < n_tokens;) {
    // as many tokens as the pool gives pages for, at most a page's worth at a time; pages behind the windows come back in between
    int m = std::min(std::min(n_tokens - i, PAGE_TOKENS), n->pool.room(seq));
    if (m < 1) return set_error(CAI_ERR_STATE, "greedy generation: the cache pool is out of pages after %d of %d tokens", i, n_tokens);
    int rc = n->pool.reserve(seq, q.len + m);
    if (rc || (rc = n->pool.upload_table())) return rc;
    for (int k = 0; k < m;) {
      const int steps = m - k >= GEN_STEPS ? GEN_STEPS : 1;
      if ((rc = run_captured(n, 1, steps, true, q.len + k + steps))) return rc;
      k += steps;
    }
    q.len += m; i += m;
    n->pool.trim(seq);
  }
  CAI_HIP(hipMemcpyAsync(out_host, n->d_gen, (size_t)n_tokens * 4, hipMemcpyDeviceToHost, st));
  CAI_HIP(hipStreamSynchronize(st));
  n->row_of.assign(1, 0); n->rows_gathered = false;
  return CAI_OK;
}

int net_len(const LayeredNet* n, int seq) { return n->pool.seq[seq].len; }
int net_room(const LayeredNet* n, int seq) { return n->pool.room(seq); }
int net_pool_pages(const LayeredNet* n) { return n->pool.n_pages; }
int net_peak_pages(const LayeredNet* n, int64_t total, int portion)
{
  if (!n->pool.n_pages) return 0;
  // a step's rows and the window before them, which may start and end inside a page
  const int64_t window = ((int64_t)n->pool.keep - 1 + portion + 2 * (PAGE_TOKENS - 1)) / PAGE_TOKENS;
  return (int)std::min<int64_t>((total + PAGE_TOKENS - 1) / PAGE_TOKENS, window);
}
int net_rows(const LayeredNet* n, int seq) { const auto& q = n->pool.seq[seq]; return n->pool.n_pages ? q.len - q.first_page * PAGE_TOKENS : 0; }
int net_n_runs(const LayeredNet* n) { return (int)n->runs.size(); }
int net_reset(LayeredNet* n, int seq) { n->pool.free_seq(seq); return CAI_OK; }
const NetSpec& net_spec(const LayeredNet* n) { return n->s; }
float* net_logits(LayeredNet* n, int row) { return row >= 0 && row < (int)n->row_of.size() ? n->logits + (size_t)n->row_of[row] * n->s.vocab : nullptr; }

int net_fork(LayeredNet* n, int src, int dst)
{
  if (src == dst) return CAI_OK;
  const int rc = n->pool.fork(src, dst);
  if (rc) { n->pool.free_seq(dst); return rc; }
  CAI_HIP(hipStreamSynchronize(ctx().stream));
  return CAI_OK;
}

int net_hidden(LayeredNet* n, int row, float* host)
{
  if (row < 0 || row >= (int)n->row_of.size()) return set_error(CAI_ERR_STATE, "hidden state: row %d of the last step's %zu rows with logits", row, n->row_of.size());
  const char* src = (const char*)(n->rows_gathered ? n->hw : n->h) + (size_t)n->row_of[row] * n->wp * n->es;
  std::vector<uint32_t> raw(n->s.width);
  CAI_HIP(hipMemcpyAsync(raw.data(), src, (size_t)n->s.width * n->es, hipMemcpyDeviceToHost, ctx().stream));
  CAI_HIP(hipStreamSynchronize(ctx().stream));
  if (n->es == 4) memcpy(host, raw.data(), (size_t)n->s.width * 4);
  else { const uint16_t* b = (const uint16_t*)raw.data(); for (int i = 0; i < n->s.width; i++) { const uint32_t u = (uint32_t)b[i] << 16; memcpy(host + i, &u, 4); } }
  return CAI_OK;
}

int64_t net_weight_bytes(const LayeredNet* n)
{
  // a layer that runs several times is streamed as often
  auto qb = [](const cai_qw_s* w) { return w ? w->algo_bytes : 0; };
  int64_t b = qb(n->s.head) + n->s.embed->algo_bytes / n->s.embed->rows + 2 * (int64_t)n->s.width * 4;
  for (const NetRun& r : n->runs) {
    const NetLayer& y = n->s.layers[r.layer];
    const NetExperts& x = y.experts;
    b += qb(y.in) + qb(y.delta.out) + qb(y.latent.uq) + qb(y.latent.up) + qb(y.latent.out) + qb(y.gla.out) + qb(y.attn.out) + qb(y.ssd.out) + qb(y.delta.w.a2) + qb(y.delta.w.g2) + qb(y.gateup) + qb(y.down) + qb(y.in2) + 8 * (int64_t)n->s.width * 4;
    if (r.enter) b += qb(n->s.loop_in);
    if (x.n) b += qb(x.router) + qb(x.s_gateup) + qb(x.s_down) + (qb(x.gateup) + qb(x.down)) / x.n * x.top;   // (of one token)
  }
  return b;
}

// ------------------------------------------------------------------------------------------
// snapshots: live pages and state of one sequence
// ------------------------------------------------------------------------------------------
struct NetSnap {
  int len = 0, first_page = 0, end_page = 0, n_attn = 0, n_state = 0; int64_t bytes = 0;
  char* data = nullptr;
};
static int64_t snap_bytes(const LayeredNet* n, int pages)
{
  int64_t b = 0;
  for (auto& a : n->pool.attn) b += pages * a.page_elems * (int64_t)n->es;
  for (auto& d : n->pool.state) b += (d.s_elems + d.h_elems) * 4;
  return b;
}
// walks the pieces of a sequence in snapshot order: f(device pointer, bytes, offset)
template <typename F> static int snap_walk(LayeredNet* n, int seq, F f)
{
  int64_t off = 0; int rc;
  const auto& q = n->pool.seq[seq];
  for (int p = q.first_page; n->pool.n_pages && p < q.end_page; p++)
    for (auto& a : n->pool.attn) {
      const size_t sz = (size_t)a.page_elems * n->es;
      if ((rc = f((char*)a.base + n->pool.table[(size_t)seq * n->pool.n_pages + p % n->pool.n_pages] * sz, sz, off))) return rc;
      off += sz;
    }
  for (auto& d : n->pool.state) {
    if (d.s_elems && (rc = f((char*)(d.S + seq * d.s_elems), (size_t)d.s_elems * 4, off))) return rc;
    off += d.s_elems * 4;
    if (d.h_elems && (rc = f((char*)(d.hist + seq * d.h_elems), (size_t)d.h_elems * 4, off))) return rc;
    off += d.h_elems * 4;
  }
  return CAI_OK;
}
int net_snapshot(LayeredNet* n, int seq, NetSnap** out)
{
  const auto& q = n->pool.seq[seq];
  NetSnap* s = new NetSnap();
  s->len = q.len; s->first_page = q.first_page; s->end_page = q.end_page; s->n_attn = (int)n->pool.attn.size(); s->n_state = (int)n->pool.state.size();
  s->bytes = snap_bytes(n, q.end_page - q.first_page);
  if (hipMalloc((void**)&s->data, (size_t)s->bytes) != hipSuccess) { (void)hipGetLastError(); delete s; return set_error(CAI_ERR_NOMEM, "snapshot: out of device memory (a sequence of %d tokens)", q.len); }
  const int rc = snap_walk(n, seq, [&](char* p, size_t sz, int64_t off) -> int { CAI_HIP(hipMemcpyAsync(s->data + off, p, sz, hipMemcpyDeviceToDevice, ctx().stream)); return CAI_OK; });
  if (rc) { net_snap_free(s); return rc; }
  CAI_HIP(hipStreamSynchronize(ctx().stream));
  *out = s;
  return CAI_OK;
}
int net_restore(LayeredNet* n, int seq, const NetSnap* s)
{
  const int pages = s->end_page - s->first_page;
  CAI_REQUIRE(s->n_attn == (int)n->pool.attn.size() && s->n_state == (int)n->pool.state.size() && s->bytes == snap_bytes(n, pages), "restore: the snapshot is of another model");
  n->pool.free_seq(seq);
  auto& q = n->pool.seq[seq];
  q.first_page = q.end_page = s->first_page;
  int rc = n->pool.reserve(seq, s->end_page * PAGE_TOKENS);
  if (rc) { q = SeqPool::Seq(); return rc; }
  q.len = s->len;
  rc = snap_walk(n, seq, [&](char* p, size_t sz, int64_t off) -> int { CAI_HIP(hipMemcpyAsync(p, s->data + off, sz, hipMemcpyDeviceToDevice, ctx().stream)); return CAI_OK; });
  if (rc) return rc;
  CAI_HIP(hipStreamSynchronize(ctx().stream));
  return CAI_OK;
}
void net_snap_free(NetSnap* s) { if (!s) return; if (s->data) (void)hipFree(s->data); delete s; }

}  // namespace cai
