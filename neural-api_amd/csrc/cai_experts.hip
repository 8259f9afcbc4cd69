// Mixtures of experts over bfloat16 weights: routing, gathering kernels for a few rows (decode), grouped products for more.
//
// The experts' gated matrices lie one after the other in one bank, and so do their output matrices.  A chosen expert's weight
// multiplies its gated activations, which the output product is linear in, so that the sum over a row's experts is one long product.
// Experts without a gate have one matrix and an activation in the gated one's place.  Everything about the routing is 32-bit.
#include "cai_lin_epilogue.hpp"

#include <algorithm>

namespace cai {

// maximum over a wave, and minimum of whole numbers, in every lane (a lane without a partner meets itself)
template <int CTRL, int ROWS> __device__ __forceinline__ float dpp_max(float v)
{
  const int x = __builtin_bit_cast(int, v);
  return fmaxf(v, __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(x, x, CTRL, ROWS, 0xf, false)));
}
template <int CTRL, int ROWS> __device__ __forceinline__ int dpp_min(int v) { return min(v, __builtin_amdgcn_update_dpp(v, v, CTRL, ROWS, 0xf, false)); }
__device__ __forceinline__ float wave_max(float v)
{
  v = dpp_max<0x111, 0xf>(v); v = dpp_max<0x112, 0xf>(v); v = dpp_max<0x114, 0xf>(v); v = dpp_max<0x118, 0xf>(v); v = dpp_max<0x142, 0xa>(v); v = dpp_max<0x143, 0xc>(v);
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), 63));
}
__device__ __forceinline__ int wave_min(int v)
{
  v = dpp_min<0x111, 0xf>(v); v = dpp_min<0x112, 0xf>(v); v = dpp_min<0x114, 0xf>(v); v = dpp_min<0x118, 0xf>(v); v = dpp_min<0x142, 0xa>(v); v = dpp_min<0x143, 0xc>(v);
  return __builtin_amdgcn_readlane(v, 63);
}
// a finished sum over the lanes of a wave, in every lane
__device__ __forceinline__ float lanes_total(float v)
{
  v = wave_sum(v);
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), 63));
}

// How a row's experts are chosen and weighted.
struct Routing { const float* correction; int n, top, route; float scale; int groups, keep, per_group; };

__device__ __forceinline__ float route_sigmoid(float z)
{
  if (z >= 0.0f) return 1.0f / (1.0f + expf(-z));
  const float s = expf(z); return s / (1.0f + s);
}

// how many of the first n lanes hold more, or as much in front of this lane
__device__ __forceinline__ int lane_rank(float v, int n, int lane)
{
  int rank = 0;
  for (int j0 = 0; j0 < n; j0 += 8)
#pragma unroll
    for (int u = 0; u < 8; u++) {          // (n is 64 at most; lanes past it do not count)
      const int j = j0 + u;
      const float o = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), j));
      rank += j < n && (o > v || (o == v && j < lane));
    }
  return rank;
}

// One row's experts (SIG: by ROUTE_SIGMOID), by one wave: lane k < top ends with the k-th choice and its weight.  Equal choice scores: the lower index.
template <bool SIG>
__device__ __forceinline__ void route_row(const float* z, const Routing& q, const int lane, int& expert, float& weight)
{
  const float* correction = q.correction;
  const int n = q.n, top = q.top;
  constexpr int PER = EXPERTS_MAX / 64;
  float s[PER], c[PER], m = -INFINITY, sum = 0.0f;
#pragma unroll
  for (int i = 0; i < PER; i++) { const int e = lane + 64 * i; s[i] = e < n ? z[e] : -INFINITY; c[i] = e < n && correction ? correction[e] : 0.0f; m = fmaxf(m, s[i]); }
  uint64_t kept = ~0ull;                   // groups that take part
  const int per_group = q.per_group;
  if constexpr (SIG) {
#pragma unroll
    for (int i = 0; i < PER; i++) if (64 * i < n) s[i] = route_sigmoid(s[i]);
    if (q.keep < q.groups) {               // a lane a group: its two largest choice scores, and how many groups are better
      float a = -INFINITY, b = -INFINITY;
      auto meet = [&](float v) { b = fmaxf(b, fminf(a, v)); a = fmaxf(a, v); };
      if (n <= 64) {
        const float v = s[0] + c[0];
        for (int i0 = 0; i0 < per_group; i0 += 4)
#pragma unroll
          for (int i = i0; i < i0 + 4; i++) { const float o = __shfl(v, (lane * per_group + i) & 63); meet(i < per_group ? o : -INFINITY); }
      } else if (lane < q.groups)
#pragma unroll 4
        for (int i = 0; i < per_group; i++) {
          const int e = lane * per_group + i;
          meet(route_sigmoid(z[e]) + (correction ? correction[e] : 0.0f));
        }
      const float score = per_group > 1 ? a + b : a;
      kept = __ballot(lane < q.groups && lane_rank(score, q.groups, lane) < q.keep);
    }
  } else m = wave_max(m);
  if (!SIG && q.route == ROUTE_ALL) {
#pragma unroll
    for (int i = 0; i < PER; i++) if (64 * i < n) { s[i] = expf(s[i] - m); sum += s[i]; }
    sum = lanes_total(sum);
  }
#pragma unroll
  for (int i = 0; i < PER; i++) {
    if (!SIG && 64 * i < n && q.route == ROUTE_ALL) s[i] /= sum;
    bool in = lane + 64 * i < n;
    if (SIG && 64 * i < n) in = in && (kept >> ((lane + 64 * i) / per_group & 63) & 1);
    c[i] = in ? s[i] + c[i] : -INFINITY;
  }
  if (SIG && n <= 64) {                    // a lane an expert: each goes to the lane of its rank
    const int to = (lane < n ? lane_rank(c[0], n, lane) : lane) * 4;
    expert = min(max(__builtin_amdgcn_ds_permute(to, lane), 0), n - 1);
    weight = __builtin_bit_cast(float, __builtin_amdgcn_ds_permute(to, __builtin_bit_cast(int, s[0]))) * q.scale;
    return;
  }
  expert = 0; weight = 0.0f;
  float total = 0.0f;
  for (int k = 0; k < top; k++) {
    float bv = -INFINITY, bs = 0.0f; int be = n - 1;     // (always a valid expert, also if the scores are not numbers)
#pragma unroll
    for (int i = 0; i < PER; i++) if (64 * i < n && c[i] > bv) { bv = c[i]; be = lane + 64 * i; bs = s[i]; }
    const float most = wave_max(bv);
    be = wave_min(bv == most ? be : n - 1);
    bs = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, bs), be & 63));
    if (!SIG && q.route == ROUTE_AMONG) bs = expf(bs - m);       // (m is the largest logit, the first choice)
    total += bs;
    if (lane == k) { expert = be; weight = bs; }
#pragma unroll
    for (int i = 0; i < PER; i++) if (lane + 64 * i == be) c[i] = -INFINITY;
  }
  weight = SIG ? weight * q.scale : weight / (total + 1e-20f) * q.scale;
}

// eight activations times eight weights
template <typename AT> __device__ __forceinline__ float dot8(const AT* x, const u32x4 w, float s)
{
  if constexpr (sizeof(AT) == 2) {
    const u32x4 a = *reinterpret_cast<const u32x4*>(x);
#pragma unroll
    for (int j = 0; j < 4; j++) { s = fmaf(bf16_lo(w[j]), bf16_lo(a[j]), s); s = fmaf(bf16_hi(w[j]), bf16_hi(a[j]), s); }
  } else {
    const f32x4 a = *reinterpret_cast<const f32x4*>(x), b = *reinterpret_cast<const f32x4*>(x + 4);
    s = fmaf(bf16_lo(w[0]), a[0], s); s = fmaf(bf16_hi(w[0]), a[1], s); s = fmaf(bf16_lo(w[1]), a[2], s); s = fmaf(bf16_hi(w[1]), a[3], s);
    s = fmaf(bf16_lo(w[2]), b[0], s); s = fmaf(bf16_hi(w[2]), b[1], s); s = fmaf(bf16_lo(w[3]), b[2], s); s = fmaf(bf16_hi(w[3]), b[3], s);
  }
  return s;
}

// ------------------------------------------------------------------------------------------
// Up to EXPERTS_FEW rows.  The gate and up kernel takes blockIdx x = outputs, y = entry; a wave makes two outputs of every row of its
// entry, so that a matrix is read once however many rows chose it.  The entries of one row are its choices, and every wave routes the
// row itself; for more rows a launch before it routes them and lists the experts that were chosen.  The last entry is the shared one.
// Experts that are not gated: four outputs a wave.
// ------------------------------------------------------------------------------------------
struct FewEntry { int32_t expert, n_rows; uint8_t row[EXPERTS_FEW], slot[EXPERTS_FEW]; };
static_assert(sizeof(FewEntry) == EXPERTS_FEW_WORDS * 4, "size of a listed expert");
struct FewGateUp {
  const uint16_t *w, *ws; int ldw, gu_rows; Routing q; int ff, ff_s; float limit, limit_s; int glu, glu_s; int mid_p, active; int n_rows; int act;
};

template <bool SIG>
__global__ __launch_bounds__(64 * EXPERTS_FEW) void experts_few_kernel(const float* z, const int64_t ldz, const Routing q, const int n_rows, float* wgt, FewEntry* list, int32_t* n_list)
{
  const int n = q.n, top = q.top;
  __shared__ __align__(4) int8_t slot_of[EXPERTS_FEW][EXPERTS_MAX];   // the choice of a row that is this expert, -1: none
  __shared__ int wave_count[EXPERTS_FEW];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, tid = threadIdx.x;
  for (int i = tid; i < EXPERTS_FEW * EXPERTS_MAX / 4; i += 64 * EXPERTS_FEW) reinterpret_cast<int32_t*>(&slot_of[0][0])[i] = -1;
  __syncthreads();
  if (wave < n_rows) {
    int e; float w;
    route_row<SIG>(z + wave * ldz, q, lane, e, w);
    if (lane < top) { wgt[wave * top + lane] = w; slot_of[wave][e] = (int8_t)lane; }
  }
  __syncthreads();
  // a thread per expert: the chosen ones in order
  static_assert(64 * EXPERTS_FEW >= EXPERTS_MAX, "a thread per expert");
  FewEntry x{tid, 0, {}, {}};
  if (tid < n)
#pragma unroll
    for (int r = 0; r < EXPERTS_FEW; r++)
      if (slot_of[r][tid] >= 0) { x.row[x.n_rows] = (uint8_t)r; x.slot[x.n_rows] = (uint8_t)slot_of[r][tid]; x.n_rows++; }
  const uint64_t chosen = __ballot(x.n_rows > 0);
  if (lane == 0) wave_count[wave] = __popcll(chosen);
  __syncthreads();
  int at = __popcll(chosen & ((1ull << lane) - 1)), total = 0;
  for (int i = 0; i < EXPERTS_FEW; i++) { if (i < wave) at += wave_count[i]; total += wave_count[i]; }
  if (x.n_rows) list[at] = x;
  if (tid == 0) *n_list = total;
}

template <typename AT, int NB, bool GATED, bool SIG>       // (SIG counts for one row only)
__global__ __launch_bounds__(256) void experts_gateup_kernel(const FewGateUp p, const float* z, const float* wgt, const FewEntry* list, const int32_t* n_list, const AT* h, const int64_t ldh, int32_t* sel, AT* mid)
{
  constexpr int UNROLL = NB == 1 ? 2 : 1;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), entry = blockIdx.y;
  const bool shared = p.ws && entry == (int)gridDim.y - 1;
  constexpr int OUT = GATED ? 2 : 4;
  const int ff = shared ? p.ff_s : p.ff, j0 = (blockIdx.x * 4 + wave) * OUT;
  if (j0 >= ff) return;
  const uint16_t* W = p.ws;
  float weight = 1.0f;
  int nb = p.n_rows;
  if (!shared) {
    if constexpr (NB == 1) {
      int e; float wt;
      route_row<SIG>(z, p.q, lane, e, wt);
      if (j0 == 0 && lane == entry) sel[entry] = e;
      W = p.w + (int64_t)__shfl(e, entry) * p.gu_rows * p.ldw; weight = __shfl(wt, entry);
    } else {
      if (entry >= *n_list) return;
      W = p.w + (int64_t)list[entry].expert * p.gu_rows * p.ldw; nb = list[entry].n_rows;
    }
  }
  const int j1 = min(j0 + 1, ff - 1);
  const uint16_t* wr[4];
#pragma unroll
  for (int i = 0; i < 4; i++) wr[i] = W + (int64_t)(GATED ? glu_row(i < 2 ? j0 : j1, i & 1) : min(j0 + i, ff - 1)) * p.ldw;
  const AT* x[NB];
#pragma unroll
  for (int b = 0; b < NB; b++) x[b] = h + (int64_t)(NB == 1 || b >= nb ? 0 : shared ? b : list[entry].row[b]) * ldh;
  float acc[NB][4];
#pragma unroll
  for (int b = 0; b < NB; b++)
#pragma unroll
    for (int i = 0; i < 4; i++) acc[b][i] = 0.0f;
#pragma unroll UNROLL
  for (int k = lane * 8; k < p.ldw; k += 512) {
    u32x4 v[4];
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = *reinterpret_cast<const u32x4*>(wr[i] + k);
#pragma unroll
    for (int b = 0; b < NB; b++) {
      if (b >= nb) break;
#pragma unroll
      for (int i = 0; i < 4; i++) acc[b][i] = dot8<AT>(x[b] + k, v[i], acc[b][i]);
    }
  }
#pragma unroll
  for (int b = 0; b < NB; b++) {
    if (b >= nb) break;
#pragma unroll
    for (int i = 0; i < 4; i++) acc[b][i] = lanes_total(acc[b][i]);
    const int row = NB == 1 ? 0 : shared ? b : list[entry].row[b], slot = NB == 1 ? entry : shared ? p.q.top : list[entry].slot[b];
    if (NB > 1) weight = shared ? 1.0f : wgt[row * p.q.top + slot];
    if constexpr (!GATED) {
      if (lane < 4 && j0 + lane < ff)
        put_act<AT>(mid, (int64_t)row * p.active + slot * p.mid_p + j0 + lane, lin_act(lane & 2 ? (lane & 1 ? acc[b][3] : acc[b][2]) : lane & 1 ? acc[b][1] : acc[b][0], p.act, 0.0f) * weight);
    } else if (lane < 2 && j0 + lane < ff)
      put_act<AT>(mid, (int64_t)row * p.active + slot * p.mid_p + j0 + lane,
                  glu_pair(shared ? p.glu_s : p.glu, shared ? p.limit_s : p.limit, lane ? acc[b][2] : acc[b][0], lane ? acc[b][3] : acc[b][1]) * weight);
  }
}

// The output product of one row: a wave makes two outputs over all choices, then the residual update.  wo: the product beside (null:
// none).
struct BesideArg { const uint16_t* w = nullptr; const void* x = nullptr; int ld = 0; int64_t ldx = 0; LinEpi e; };
template <typename AT>
__global__ __launch_bounds__(256) void experts_down_kernel(const uint16_t* w, const uint16_t* ws, const int ldw, const int lds, const int top, const int width, const int n_experts,
                                                           const int32_t* sel, const AT* mid, const LinEpi e, const BesideArg o)
{
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int o0 = (blockIdx.x * 4 + wave) * 2;
  if (o0 >= width) return;
  const int o1 = min(o0 + 1, width - 1);
  float acc[2] = {0.0f, 0.0f};
  const AT* x = mid;
  float b0 = 0.0f, b1 = 0.0f;
  auto slot = [&](const uint16_t* m, int ld) {
    const uint16_t *a = m + (int64_t)o0 * ld, *b = m + (int64_t)o1 * ld;
#pragma unroll 2
    for (int k = lane * 8; k < ld; k += 512) {
      const u32x4 va = *reinterpret_cast<const u32x4*>(a + k), vb = *reinterpret_cast<const u32x4*>(b + k);
      acc[0] = dot8<AT>(x + k, va, acc[0]); acc[1] = dot8<AT>(x + k, vb, acc[1]);
    }
    x += ld;
  };
  if (o.w) {
    x = reinterpret_cast<const AT*>(o.x);
    slot(o.w, o.ld);
    b0 = lanes_total(acc[0]); b1 = lanes_total(acc[1]);
    acc[0] = acc[1] = 0.0f;
    x = mid;
  }
#pragma unroll 4
  for (int s = 0; s < top; s++) slot(w + (int64_t)min(max(sel[s], 0), n_experts - 1) * width * ldw, ldw);
  if (ws) slot(ws, lds);
  const float y0 = lanes_total(acc[0]), y1 = lanes_total(acc[1]);
  if (lane < 2 && o0 + lane < width) {
    if (o.w) join_two(o.e, lane ? b1 : b0, e, lane ? y1 : y0, o0 + lane, 0);
    else epi_one<AT>(e, o0 + lane, 0, lane ? y1 : y0);
  }
}

// That of several rows, an entry at a time (blockIdx as in the gate and up kernel): outputs of every choice, summed by experts_sum_kernel.
// The product beside takes the place of the shared expert: ws over rows xs, lxs apart.
template <typename AT, int NB>
__global__ __launch_bounds__(256) void experts_out_kernel(const uint16_t* w, const uint16_t* ws, const int ldw, const int lds, const int top, const int active, const int width, const int n_rows,
                                                          const FewEntry* list, const int32_t* n_list, const AT* mid, float* y, float* ys, const AT* xs, const int64_t lxs)
{
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), entry = blockIdx.y;
  const bool shared = ws && entry == (int)gridDim.y - 1;
  const int o0 = (blockIdx.x * 4 + wave) * 2;
  if (o0 >= width || (!shared && entry >= *n_list)) return;
  const int o1 = min(o0 + 1, width - 1), ld = shared ? lds : ldw, nb = shared ? n_rows : list[entry].n_rows;
  const uint16_t* m = shared ? ws : w + (int64_t)list[entry].expert * width * ldw;
  const uint16_t *wa = m + (int64_t)o0 * ld, *wb = m + (int64_t)o1 * ld;
  int row[NB], slot[NB];
  const AT* x[NB];
  float acc[NB][2];
#pragma unroll
  for (int b = 0; b < NB; b++) {
    row[b] = b >= nb ? 0 : shared ? b : list[entry].row[b]; slot[b] = b >= nb ? 0 : shared ? top : list[entry].slot[b];
    x[b] = shared && xs ? xs + row[b] * lxs : mid + (int64_t)row[b] * active + slot[b] * ldw;
    acc[b][0] = acc[b][1] = 0.0f;
  }
  for (int k = lane * 8; k < ld; k += 512) {
    const u32x4 va = *reinterpret_cast<const u32x4*>(wa + k), vb = *reinterpret_cast<const u32x4*>(wb + k);
#pragma unroll
    for (int b = 0; b < NB; b++) {
      if (b >= nb) break;
      acc[b][0] = dot8<AT>(x[b] + k, va, acc[b][0]); acc[b][1] = dot8<AT>(x[b] + k, vb, acc[b][1]);
    }
  }
#pragma unroll
  for (int b = 0; b < NB; b++) {
    if (b >= nb) break;
    const float y0 = lanes_total(acc[b][0]), y1 = lanes_total(acc[b][1]);
    if (lane < 2 && o0 + lane < width) (shared ? ys + (int64_t)row[b] * width : y + ((int64_t)row[b] * top + slot[b]) * width)[o0 + lane] = lane ? y1 : y0;
  }
}

// ------------------------------------------------------------------------------------------
// More rows: routing (a wave a row), the (row, choice) pairs ordered by expert with their tiles (one work-group), grouped products
// (cai_linear_bf16.hip), and the sum of a row's outputs with the residual update.
// ------------------------------------------------------------------------------------------
// Router scores of 16 rows and their choices: sixteen waves share the width, 16 ET experts at a time; the matrix cores multiply as in the
// other products (bfloat16, or exactly widened weights in 32-bit), the sums meet in LDS.
constexpr int ROUTE_WAVES = 16;
template <typename AT, int ET, bool SIG>
__global__ __launch_bounds__(64 * ROUTE_WAVES) void experts_route_kernel(const uint16_t* W, const int ldw, const AT* h, const int64_t ldh, const Routing q, const int n_rows, int32_t* sel, float* wgt)
{
  const int n = q.n, top = q.top;
  extern __shared__ float lds[];                         // [ROUTE_WAVES][16 ET][16] sums, [16][n] scores
  constexpr int STEP = sizeof(AT) == 2 ? 32 : 16, AHEAD = 8;
  float* z = lds + ROUTE_WAVES * 16 * ET * 16;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), fr = lane & 15, fg = lane >> 4, r0 = blockIdx.x * 16;
  const AT* xp = h + (int64_t)min(r0 + fr, n_rows - 1) * ldh + fg * (STEP / 4);
  for (int e0 = 0; e0 < n; e0 += 16 * ET) {
    const uint16_t* wp[ET]; f32x4 acc[ET];
#pragma unroll
    for (int t = 0; t < ET; t++) { wp[t] = W + (int64_t)min(e0 + t * 16 + fr, n - 1) * ldw + fg * (STEP / 4); acc[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f}; }
    for (int k0 = wave * STEP; k0 < ldw; k0 += ROUTE_WAVES * STEP * AHEAD) {
      u32x4 x[AHEAD], wv[AHEAD][ET];
#pragma unroll
      for (int a = 0; a < AHEAD; a++) {                  // (turns past the width repeat the first one and are not used)
        const int k = k0 + a * ROUTE_WAVES * STEP < ldw ? k0 + a * ROUTE_WAVES * STEP : k0;
        x[a] = *reinterpret_cast<const u32x4*>(xp + k);
#pragma unroll
        for (int t = 0; t < ET; t++) {
          if constexpr (sizeof(AT) == 2) wv[a][t] = *reinterpret_cast<const u32x4*>(wp[t] + k);
          else { const uint2 u = *reinterpret_cast<const uint2*>(wp[t] + k); wv[a][t] = u32x4{u.x << 16, u.x & 0xffff0000u, u.y << 16, u.y & 0xffff0000u}; }
        }
      }
#pragma unroll
      for (int a = 0; a < AHEAD; a++) {
        if (k0 + a * ROUTE_WAVES * STEP >= ldw) continue;
#pragma unroll
        for (int t = 0; t < ET; t++) {
          if constexpr (sizeof(AT) == 2) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wv[a][t]), __builtin_bit_cast(bf16x8, x[a]), acc[t], 0, 0, 0);
          else {
            const f32x4 wf = __builtin_bit_cast(f32x4, wv[a][t]), xf = __builtin_bit_cast(f32x4, x[a]);
#pragma unroll
            for (int q = 0; q < 4; q++) acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(wf[q], xf[q], acc[t], 0, 0, 0);
          }
        }
      }
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < ET; t++)
#pragma unroll
      for (int i = 0; i < 4; i++) lds[(wave * 16 * ET + t * 16 + fg * 4 + i) * 16 + fr] = acc[t][i];
    __syncthreads();
    for (int i = tid; i < 16 * 16 * ET; i += 64 * ROUTE_WAVES) {
      const int e = i >> 4, r = i & 15;
      float s = 0.0f;
#pragma unroll
      for (int v = 0; v < ROUTE_WAVES; v++) s += lds[(v * 16 * ET + e) * 16 + r];
      if (e0 + e < n) z[r * n + e0 + e] = s;
    }
  }
  __syncthreads();
  for (int r = wave; r < 16 && r0 + r < n_rows; r += ROUTE_WAVES) {
    int e; float w;
    route_row<SIG>(z + r * n, q, lane, e, w);
    if (lane < top) { sel[(int64_t)(r0 + r) * top + lane] = e; wgt[(int64_t)(r0 + r) * top + lane] = w; }
  }
}

// choices of rows whose logits are there already, a wave a row
template <bool SIG>
__global__ __launch_bounds__(256) void experts_pick_kernel(const float* z, const int64_t ldz, const Routing q, const int n_rows, int32_t* sel, float* wgt)
{
  const int lane = threadIdx.x & 63;
  const int64_t row = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= n_rows) return;
  int e; float w;
  route_row<SIG>(z + row * ldz, q, lane, e, w);
  if (lane < q.top) { sel[row * q.top + lane] = e; wgt[row * q.top + lane] = w; }
}

__global__ __launch_bounds__(1024) void experts_order_kernel(const int32_t* sel, const int n, const int pairs, const int tile, int32_t* order, int32_t* tiles, int32_t* n_tiles)
{
  __shared__ int count[EXPERTS_MAX], at[EXPERTS_MAX], tile0[EXPERTS_MAX];
  const int tid = threadIdx.x;
  for (int e = tid; e < n; e += 1024) count[e] = 0;
  __syncthreads();
  for (int i = tid; i < pairs; i += 1024) atomicAdd(&count[sel[i]], 1);
  __syncthreads();
  if (tid < 64) {                          // running sums of counts and tiles over the experts, a wave
    int base = 0, tbase = 0;
    for (int e0 = 0; e0 < n; e0 += 64) {
      const int e = e0 + tid, c = e < n ? count[e] : 0, t = (c + tile - 1) / tile;
      int a = c, b = t;
      for (int o = 1; o < 64; o <<= 1) { const int x = __shfl_up(a, o), y = __shfl_up(b, o); if (tid >= o) { a += x; b += y; } }
      if (e < n) { at[e] = base + a - c; tile0[e] = tbase + b - t; }
      base += __shfl(a, 63); tbase += __shfl(b, 63);
    }
    if (tid == 0) *n_tiles = tbase;
  }
  __syncthreads();
  for (int e = tid; e < n; e += 1024) {
    int t = tile0[e];
    for (int c = 0; c < count[e]; c += tile, t++) { tiles[3 * t] = e; tiles[3 * t + 1] = at[e] + c; tiles[3 * t + 2] = min(tile, count[e] - c); }
  }
  __syncthreads();
  for (int i = tid; i < pairs; i += 1024) order[atomicAdd(&at[sel[i]], 1)] = i;
}

template <typename AT>
__global__ __launch_bounds__(256) void experts_sum_kernel(const float* y, const float* ys, const int top, const int width, const LinEpi e, const LinEpi beside)
{
  const int64_t row = blockIdx.y;
  for (int i = blockIdx.x * 256 + threadIdx.x; i < width; i += gridDim.x * 256) {
    const float s0 = ys ? ys[row * width + i] : 0.0f;
    float s = beside.y ? 0.0f : s0;
#pragma unroll 4
    for (int k = 0; k < top; k++) s += y[(row * top + k) * width + i];
    if (beside.y) join_two(beside, s0, e, s, i, row);
    else epi_one<AT>(e, i, (int)row, s);
  }
}

static Routing routing(const NetExperts& x) { return Routing{x.correction, x.n, x.top, x.route, x.scale, x.groups, x.keep, x.n / x.groups}; }

template <typename AT, int NB>
static void run_few(const NetExperts& x, int width, const AT* h, int64_t ldh, int n_rows, const float* z, int64_t ldz, const ExpertBuf& b, const LinEpi& res, const BesideLin* beside)
{
  auto st = ctx().stream;
  const uint16_t *sg = x.s_gateup ? (const uint16_t*)x.s_gateup->data : nullptr, *sd = x.s_down ? (const uint16_t*)x.s_down->data : nullptr;
  const FewGateUp p{(const uint16_t*)x.gateup->data, sg, (int)x.gateup->ld, x.gu_rows(), routing(x), x.ff, x.ff_shared,
                    x.limit, x.limit_shared, x.glu, x.glu_shared, x.mid_p(), x.active(), n_rows, x.act};
  FewEntry* list = (FewEntry*)b.few;
  const bool sig = x.route == ROUTE_SIGMOID;
  if (NB > 1) hipLaunchKernelGGL(sig ? experts_few_kernel<true> : experts_few_kernel<false>, dim3(1), dim3(64 * EXPERTS_FEW), 0, st, z, ldz, p.q, n_rows, b.wgt, list, b.n_tiles);
  const int entries = NB == 1 ? x.top : std::min(x.n, n_rows * x.top);
  const dim3 mids(x.gated ? (std::max(x.ff, x.ff_shared) + 7) / 8 : (x.ff + 15) / 16, entries + (sg ? 1 : 0));
#define GATEUP(G, S) hipLaunchKernelGGL((experts_gateup_kernel<AT, NB, G, S>), mids, dim3(256), 0, st, p, z, b.wgt, list, b.n_tiles, h, ldh, b.sel, (AT*)b.mid)
  if (NB == 1 && sig) { if (x.gated) GATEUP(true, NB == 1); else GATEUP(false, NB == 1); }
  else if (x.gated) GATEUP(true, false); else GATEUP(false, false);
#undef GATEUP
  BesideArg o;
  if (beside) { o.w = (const uint16_t*)beside->w->data; o.x = beside->x; o.ld = (int)beside->w->ld; o.ldx = beside->ldx; o.e = beside->e; }
  const int lds = x.s_down ? (int)x.s_down->ld : 0;
  const dim3 outs((width + 7) / 8, NB == 1 ? 1 : entries + (sd || beside ? 1 : 0));
  if constexpr (NB == 1)
  {
    LinEpi e = res;
    if (!e.y) { e.y = b.y; e.ldy = width; }
    hipLaunchKernelGGL(experts_down_kernel<AT>, outs, dim3(256), 0, st, (const uint16_t*)x.down->data, sd, (int)x.down->ld, lds, x.top, width, x.n, b.sel, (const AT*)b.mid, e, o);
  }
  else {
    hipLaunchKernelGGL((experts_out_kernel<AT, NB>), outs, dim3(256), 0, st, (const uint16_t*)x.down->data, beside ? o.w : sd, (int)x.down->ld, beside ? o.ld : lds, x.top, x.active(), width, n_rows, list, b.n_tiles, (const AT*)b.mid, b.y, b.ys,
                       (const AT*)o.x, o.ldx);
    if (res.y) hipLaunchKernelGGL(experts_sum_kernel<AT>, dim3(std::min((width + 255) / 256, 32), n_rows), dim3(256), 0, st, b.y, sd || beside ? b.ys : nullptr, x.top, width, res, o.e);
  }
}

template <typename AT>
static int run(const NetExperts& x, int width, int act_t, const AT* h, int64_t ldh, int n_rows, const float* z, int64_t ldz, const ExpertBuf& b, const LinEpi& res, const BesideLin* beside)
{
  auto st = ctx().stream;
  int rc;
  if (n_rows <= EXPERTS_FEW) {
    if (!z) {
      LinEpi e; e.y = b.z; e.ldy = x.n;
      if ((rc = launch_lin(x.router, act_t, h, ldh, n_rows, e))) return rc;
      z = b.z; ldz = x.n;
    }
    if (n_rows == 1) run_few<AT, 1>(x, width, h, ldh, n_rows, z, ldz, b, res, beside);
    else if (n_rows == 2) run_few<AT, 2>(x, width, h, ldh, n_rows, z, ldz, b, res, beside);
    else if (n_rows <= 4) run_few<AT, 4>(x, width, h, ldh, n_rows, z, ldz, b, res, beside);
    else run_few<AT, 8>(x, width, h, ldh, n_rows, z, ldz, b, res, beside);
    CAI_HIP(hipGetLastError());
    return CAI_OK;
  }
  const bool sig = x.route == ROUTE_SIGMOID;
#define ROUTE(ET, S) hipLaunchKernelGGL((experts_route_kernel<AT, ET, S>), dim3((n_rows + 15) / 16), dim3(64 * ROUTE_WAVES), (ROUTE_WAVES * 16 * ET * 16 + 16 * x.n) * sizeof(float), st, \
                                        (const uint16_t*)x.router->data, (int)x.router->ld, h, ldh, routing(x), n_rows, b.sel, b.wgt)
  if (z) hipLaunchKernelGGL(sig ? experts_pick_kernel<true> : experts_pick_kernel<false>, dim3((n_rows + 3) / 4), dim3(256), 0, st, z, ldz, routing(x), n_rows, b.sel, b.wgt);
  else if (x.n <= 16) { if (sig) ROUTE(1, true); else ROUTE(1, false); }
  else if (sig) ROUTE(2, true); else ROUTE(2, false);
#undef ROUTE
  const int tile = n_rows * x.top >= x.n * 96 ? BANK_TILE_MAX : BANK_TILE;       // (by the mean number of rows of an expert)
  hipLaunchKernelGGL(experts_order_kernel, dim3(1), dim3(1024), 0, st, b.sel, x.n, n_rows * x.top, tile, b.order, b.tiles, b.n_tiles);
  BankList l{b.tiles, b.n_tiles, b.order, b.wgt, x.top, tile, x.max_tiles(n_rows, tile)};
  { LinEpi e; e.mode = x.gated ? EPI_GLU : EPI_SPLIT; e.h = b.mid; e.ldh = x.mid_p(); e.glu = x.glu; e.limit = x.limit; e.act = x.act; if ((rc = launch_lin_bank(x.gateup, x.gu_rows(), act_t, h, ldh, l, e))) return rc; }
  l.div = 0;
  { LinEpi e; e.y = b.y; e.ldy = width; if ((rc = launch_lin_bank(x.down, width, act_t, b.mid, x.mid_p(), l, e))) return rc; }
  if (x.ff_shared) {
    LinEpi e; e.mode = EPI_GLU; e.h = b.mid_s; e.ldh = x.shared_p(); e.glu = x.glu_shared; e.limit = x.limit_shared;
    if ((rc = launch_lin(x.s_gateup, act_t, h, ldh, n_rows, e))) return rc;
    LinEpi s; s.y = b.ys; s.ldy = width;
    if ((rc = launch_lin(x.s_down, act_t, b.mid_s, x.shared_p(), n_rows, s))) return rc;
  }
  if (res.y) hipLaunchKernelGGL(experts_sum_kernel<AT>, dim3(std::min((width + 255) / 256, 32), n_rows), dim3(256), 0, st, b.y, x.ff_shared ? b.ys : nullptr, x.top, width, res, LinEpi());
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int experts_run(const NetExperts& x, int width, int act_t, const void* h, int64_t ldh, int n_rows, const float* z, int64_t ldz, const ExpertBuf& b, const LinEpi& res, const BesideLin* beside)
{
  CAI_REQUIRE(!beside || (n_rows <= EXPERTS_FEW && !x.ff_shared && beside->w->rows == width && beside->e.mode == EPI_JOIN && res.mode == EPI_JOIN), "experts: a product of another kind beside them");
  CAI_REQUIRE(x.gated || !x.ff_shared, "experts: a shared one beside experts without a gate");
  CAI_REQUIRE(res.y || (res.mode == EPI_STORE && !x.ff_shared && !beside), "experts: outputs left apart with something beside them");
  CAI_REQUIRE(x.groups >= 1 && x.groups <= EXPERTS_GROUPS && x.n % x.groups == 0 && x.keep >= 1 && x.keep <= x.groups, "experts: %d of %d groups of %d", x.keep, x.groups, x.n);
  CAI_REQUIRE(z || x.router, "experts: neither logits nor a router");
  CAI_REQUIRE(x.n >= 1 && x.n <= EXPERTS_MAX && x.top >= 1 && x.top <= std::min(x.n, EXPERTS_TOP), "experts: %d of %d", x.top, x.n);
  return act_t == ACT_T_BF16 ? run<bf16_t>(x, width, act_t, (const bf16_t*)h, ldh, n_rows, z, ldz, b, res, beside) : run<float>(x, width, act_t, (const float*)h, ldh, n_rows, z, ldz, b, res, beside);
}

}  // namespace cai
