// Mixtures of experts over bfloat16 weights: routing, gathering kernels for a few rows (decode), grouped products for more.
//
// The experts' gated matrices lie one after the other in one bank, and so do their output matrices.  A chosen expert's weight
// multiplies its gated activations, which the output product is linear in, so that the sum over a row's experts is one long product.
// Everything about the routing is 32-bit.
#include "cai_lin_epilogue.hpp"

#include <algorithm>

namespace cai {

// One row's experts, by one wave: lane k < top ends with the k-th choice and its weight.  Equal choice scores: the lower index.
__device__ __forceinline__ void route_row(const float* z, const float* correction, const int n, const int top, const float scale, const int lane, int& expert, float& weight)
{
  constexpr int PER = EXPERTS_MAX / 64;
  float s[PER], c[PER], m = -INFINITY, sum = 0.0f;
#pragma unroll
  for (int i = 0; i < PER; i++) { const int e = lane + 64 * i; s[i] = e < n ? z[e] : -INFINITY; m = fmaxf(m, s[i]); }
#pragma unroll
  for (int o = 32; o; o >>= 1) m = fmaxf(m, __shfl_xor(m, o));
#pragma unroll
  for (int i = 0; i < PER; i++) { s[i] = expf(s[i] - m); sum += s[i]; }
#pragma unroll
  for (int o = 32; o; o >>= 1) sum += __shfl_xor(sum, o);
#pragma unroll
  for (int i = 0; i < PER; i++) {
    const int e = lane + 64 * i;
    s[i] /= sum;
    c[i] = e < n ? s[i] + (correction ? correction[e] : 0.0f) : -INFINITY;
  }
  expert = 0; weight = 0.0f;
  float total = 0.0f;
  for (int k = 0; k < top; k++) {
    float bv = -INFINITY, bs = 0.0f; int be = n - 1;     // (always a valid expert, also if the scores are not numbers)
#pragma unroll
    for (int i = 0; i < PER; i++) { const int e = lane + 64 * i; if (e < n && c[i] > bv) { bv = c[i]; be = e; bs = s[i]; } }
#pragma unroll
    for (int o = 32; o; o >>= 1) {
      const float ov = __shfl_xor(bv, o), os = __shfl_xor(bs, o); const int oe = __shfl_xor(be, o);
      if (ov > bv || (ov == bv && oe < be)) { bv = ov; be = oe; bs = os; }
    }
    total += bs;
    if (lane == k) { expert = be; weight = bs; }
#pragma unroll
    for (int i = 0; i < PER; i++) if (lane + 64 * i == be) c[i] = -INFINITY;
  }
  weight = weight / (total + 1e-20f) * scale;
}

// a finished sum over the lanes of a wave, in every lane
__device__ __forceinline__ float lanes_total(float v)
{
  v = wave_sum(v);
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), 63));
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
// A few rows, gate and up: blockIdx x = outputs, y = slot (the chosen experts, then the shared one), z = row.  A wave makes two outputs;
// every wave routes its row itself, and the first work-group of a slot and row leaves the choice for the output product.
// ------------------------------------------------------------------------------------------
struct FewGateUp {
  const uint16_t *w, *ws; int ldw, gu_rows; int n, top, ff, ff_s; float scale, limit, limit_s; int glu, glu_s; int mid_p, active;
};
template <typename AT>
__global__ __launch_bounds__(256) void experts_gateup_kernel(const FewGateUp p, const float* z, const float* correction, const AT* h, const int64_t ldh, int32_t* sel, AT* mid)
{
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), slot = blockIdx.y;
  const int64_t row = blockIdx.z;
  const bool shared = slot == p.top;
  const int ff = shared ? p.ff_s : p.ff, j0 = (blockIdx.x * 4 + wave) * 2;
  if (j0 >= ff) return;
  const uint16_t* W = p.ws;
  float weight = 1.0f;
  if (!shared) {
    int e; float wt;
    route_row(z + row * p.n, correction, p.n, p.top, p.scale, lane, e, wt);
    if (j0 == 0 && lane == slot) sel[row * p.top + slot] = e;
    e = __shfl(e, slot); weight = __shfl(wt, slot);
    W = p.w + (int64_t)e * p.gu_rows * p.ldw;
  }
  const int j1 = min(j0 + 1, ff - 1);
  const uint16_t* wr[4] = {W + (int64_t)glu_row(j0, 0) * p.ldw, W + (int64_t)glu_row(j0, 1) * p.ldw, W + (int64_t)glu_row(j1, 0) * p.ldw, W + (int64_t)glu_row(j1, 1) * p.ldw};
  const AT* x = h + row * ldh;
  float acc[4] = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll 2
  for (int k = lane * 8; k < p.ldw; k += 512) {
    u32x4 v[4];
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = *reinterpret_cast<const u32x4*>(wr[i] + k);
#pragma unroll
    for (int i = 0; i < 4; i++) acc[i] = dot8<AT>(x + k, v[i], acc[i]);
  }
#pragma unroll
  for (int i = 0; i < 4; i++) acc[i] = lanes_total(acc[i]);
  if (lane < 2 && j0 + lane < ff)
    put_act<AT>(mid, row * p.active + slot * p.mid_p + j0 + lane,
                glu_pair(shared ? p.glu_s : p.glu, shared ? p.limit_s : p.limit, lane ? acc[2] : acc[0], lane ? acc[3] : acc[1]) * weight);
}

// ------------------------------------------------------------------------------------------
// A few rows, output: a wave makes two outputs of a row over all its slots, then the residual update.
// ------------------------------------------------------------------------------------------
template <typename AT>
__global__ __launch_bounds__(256) void experts_down_kernel(const uint16_t* w, const uint16_t* ws, const int ldw, const int lds, const int top, const int active, const int width, const int n_experts,
                                                           const int32_t* sel, const AT* mid, const LinEpi e)
{
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int64_t row = blockIdx.y;
  const int o0 = (blockIdx.x * 4 + wave) * 2;
  if (o0 >= width) return;
  const int o1 = min(o0 + 1, width - 1);
  float acc[2] = {0.0f, 0.0f};
  const AT* x = mid + row * active;
  auto slot = [&](const uint16_t* m, int ld) {
    const uint16_t *a = m + (int64_t)o0 * ld, *b = m + (int64_t)o1 * ld;
#pragma unroll 2
    for (int k = lane * 8; k < ld; k += 512) {
      const u32x4 va = *reinterpret_cast<const u32x4*>(a + k), vb = *reinterpret_cast<const u32x4*>(b + k);
      acc[0] = dot8<AT>(x + k, va, acc[0]); acc[1] = dot8<AT>(x + k, vb, acc[1]);
    }
    x += ld;
  };
#pragma unroll 4
  for (int s = 0; s < top; s++) slot(w + (int64_t)min(max(sel[row * top + s], 0), n_experts - 1) * width * ldw, ldw);
  if (ws) slot(ws, lds);
  const float y0 = lanes_total(acc[0]), y1 = lanes_total(acc[1]);
  if (lane < 2 && o0 + lane < width) epi_one<AT>(e, o0 + lane, (int)row, lane ? y1 : y0);
}

// ------------------------------------------------------------------------------------------
// More rows: routing (a wave a row), the (row, choice) pairs ordered by expert with their tiles (one work-group), grouped products
// (cai_linear_bf16.hip), and the sum of a row's outputs with the residual update.
// ------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void experts_route_kernel(const float* z, const float* correction, const int n, const int top, const float scale, const int n_rows, int32_t* sel, float* wgt)
{
  const int lane = threadIdx.x & 63; const int64_t row = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= n_rows) return;
  int e; float w;
  route_row(z + row * n, correction, n, top, scale, lane, e, w);
  if (lane < top) { sel[row * top + lane] = e; wgt[row * top + lane] = w; }
}

__global__ __launch_bounds__(1024) void experts_order_kernel(const int32_t* sel, const int n, const int pairs, int32_t* order, int32_t* tiles, int32_t* n_tiles)
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
      const int e = e0 + tid, c = e < n ? count[e] : 0, t = (c + BANK_TILE - 1) / BANK_TILE;
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
    for (int c = 0; c < count[e]; c += BANK_TILE, t++) { tiles[3 * t] = e; tiles[3 * t + 1] = at[e] + c; tiles[3 * t + 2] = min(BANK_TILE, count[e] - c); }
  }
  __syncthreads();
  for (int i = tid; i < pairs; i += 1024) order[atomicAdd(&at[sel[i]], 1)] = i;
}

template <typename AT>
__global__ __launch_bounds__(256) void experts_sum_kernel(const float* y, const float* ys, const int top, const int width, const LinEpi e)
{
  const int64_t row = blockIdx.y;
  for (int i = blockIdx.x * 256 + threadIdx.x; i < width; i += gridDim.x * 256) {
    float s = ys ? ys[row * width + i] : 0.0f;
    for (int k = 0; k < top; k++) s += y[(row * top + k) * width + i];
    epi_one<AT>(e, i, (int)row, s);
  }
}

template <typename AT>
static int run(const NetExperts& x, int width, int act_t, const AT* h, int64_t ldh, int n_rows, const ExpertBuf& b, const LinEpi& res)
{
  auto st = ctx().stream;
  int rc;
  { LinEpi e; e.y = b.z; e.ldy = x.n; if ((rc = launch_lin(x.router, act_t, h, ldh, n_rows, e))) return rc; }
  if (n_rows <= EXPERTS_FEW) {
    const FewGateUp p{(const uint16_t*)x.gateup->data, x.s_gateup ? (const uint16_t*)x.s_gateup->data : nullptr, (int)x.gateup->ld, x.gu_rows(), x.n, x.top, x.ff, x.ff_shared,
                      x.scale, x.limit, x.limit_shared, x.glu, x.glu_shared, x.mid_p(), x.active()};
    const int ff = std::max(x.ff, x.ff_shared);
    hipLaunchKernelGGL(experts_gateup_kernel<AT>, dim3((ff + 7) / 8, x.top + (x.ff_shared ? 1 : 0), n_rows), dim3(256), 0, st, p, b.z, x.correction, h, ldh, b.sel, (AT*)b.mid);
    hipLaunchKernelGGL(experts_down_kernel<AT>, dim3((width + 7) / 8, n_rows), dim3(256), 0, st, (const uint16_t*)x.down->data, x.s_down ? (const uint16_t*)x.s_down->data : nullptr,
                       (int)x.down->ld, x.s_down ? (int)x.s_down->ld : 0, x.top, x.active(), width, x.n, b.sel, (const AT*)b.mid, res);
    CAI_HIP(hipGetLastError());
    return CAI_OK;
  }
  hipLaunchKernelGGL(experts_route_kernel, dim3((n_rows + 3) / 4), dim3(256), 0, st, b.z, x.correction, x.n, x.top, x.scale, n_rows, b.sel, b.wgt);
  hipLaunchKernelGGL(experts_order_kernel, dim3(1), dim3(1024), 0, st, b.sel, x.n, n_rows * x.top, b.order, b.tiles, b.n_tiles);
  BankList l{b.tiles, b.n_tiles, b.order, b.wgt, x.top, x.max_tiles(n_rows)};
  { LinEpi e; e.mode = EPI_GLU; e.h = b.mid; e.ldh = x.mid_p(); e.glu = x.glu; e.limit = x.limit; if ((rc = launch_lin_bank(x.gateup, x.gu_rows(), act_t, h, ldh, l, e))) return rc; }
  l.div = 0;
  { LinEpi e; e.y = b.y; e.ldy = width; if ((rc = launch_lin_bank(x.down, width, act_t, b.mid, x.mid_p(), l, e))) return rc; }
  if (x.ff_shared) {
    LinEpi e; e.mode = EPI_GLU; e.h = b.mid_s; e.ldh = x.shared_p(); e.glu = x.glu_shared; e.limit = x.limit_shared;
    if ((rc = launch_lin(x.s_gateup, act_t, h, ldh, n_rows, e))) return rc;
    LinEpi s; s.y = b.ys; s.ldy = width;
    if ((rc = launch_lin(x.s_down, act_t, b.mid_s, x.shared_p(), n_rows, s))) return rc;
  }
  hipLaunchKernelGGL(experts_sum_kernel<AT>, dim3(std::min((width + 255) / 256, 32), n_rows), dim3(256), 0, st, b.y, x.ff_shared ? b.ys : nullptr, x.top, width, res);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int experts_run(const NetExperts& x, int width, int act_t, const void* h, int64_t ldh, int n_rows, const ExpertBuf& b, const LinEpi& res)
{
  CAI_REQUIRE(x.n >= 1 && x.n <= EXPERTS_MAX && x.top >= 1 && x.top <= std::min(x.n, EXPERTS_TOP), "experts: %d of %d", x.top, x.n);
  return act_t == ACT_T_BF16 ? run<bf16_t>(x, width, act_t, (const bf16_t*)h, ldh, n_rows, b, res) : run<float>(x, width, act_t, (const float*)h, ldh, n_rows, b, res);
}

}  // namespace cai
