// The residual stream between sublayers that stand in RMS norms: the norm of a sublayer's result, its joining, the weighted average
// over the layers so far, the next sublayer's norm and the convolution over time in front of a mixer.
//
// One work-group a row keeps the row's values in registers from the first norm to the last.  A row's convolution needs the normed
// rows before it: of single tokens these are in the sequence's ring and the same launch takes them; a portion's rows leave the
// reciprocal of their root, and a second launch slides over them.  All of it is 32-bit.
#include "cai_lin_epilogue.hpp"

#include <algorithm>

namespace cai {

template <int V> struct Vec;
template <> struct Vec<4> {
  typedef f32x4 T;
  static __device__ __forceinline__ f32x4 bf(const uint16_t* p) { const uint2 u = *reinterpret_cast<const uint2*>(p); return f32x4{bf16_lo(u.x), bf16_hi(u.x), bf16_lo(u.y), bf16_hi(u.y)}; }
  static __device__ __forceinline__ float square(f32x4 v) { return fmaf(v[0], v[0], fmaf(v[1], v[1], fmaf(v[2], v[2], v[3] * v[3]))); }
  template <typename AT> static __device__ __forceinline__ void put(void* p, int64_t i, f32x4 v) { put_four<AT>(p, i, v); }
};
template <> struct Vec<1> {
  typedef float T;
  static __device__ __forceinline__ float bf(const uint16_t* p) { return __builtin_bit_cast(float, (uint32_t)*p << 16); }
  static __device__ __forceinline__ float square(float v) { return v * v; }
  template <typename AT> static __device__ __forceinline__ void put(void* p, int64_t i, float v) { put_act<AT>(p, i, v); }
};

// the sum over a work-group, in every thread
template <int THREADS> __device__ __forceinline__ float group_total(float v, float* red)
{
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 63) red[threadIdx.x >> 6] = v;
  __syncthreads();
  v = 0.0f;
#pragma unroll
  for (int i = 0; i < THREADS / 64; i++) v += red[i];
  return v;
}

struct StreamArg {                         // StreamStep with the embedding's matrix taken apart
  StreamStep s; const uint16_t* e; int lde;
};

template <typename AT, int V, int PER, int THREADS, bool SINGLE>
__global__ __launch_bounds__(THREADS) void stream_kernel(const StreamArg a, const StepRows r)
{
  typedef Vec<V> X; typedef typename X::T T;
  const StreamStep& s = a.s;
  __shared__ float red[2][THREADS / 64];
  const int64_t row = blockIdx.x;
  const int tid = threadIdx.x, w = s.width;
  float* xr = s.x + row * w;
  auto col = [&](int u) { return (tid + u * THREADS) * V; };
  auto at = [](const float* p) -> T { return *reinterpret_cast<const T*>(p); };
  T x[PER];
#pragma unroll
  for (int u = 0; u < PER; u++) {          // (columns past the width repeat its first ones and are not kept)
    const int c = col(u) < w ? col(u) : 0;
    if (a.e) x[u] = X::bf(a.e + (int64_t)r.tok[row] * a.lde + c) * s.embed_scale;
    else x[u] = at(xr + c);
  }
  if (!SINGLE && s.keep_ring && r.last[row] - (int)row < s.keep_taps) {
    const float inv = s.inv[row];
    float* ring = s.keep_ring + r.slot[row] * s.keep_elems + (int64_t)(r.pos[row] % s.keep_taps) * w;
#pragma unroll
    for (int u = 0; u < PER; u++) if (col(u) < w) *reinterpret_cast<T*>(ring + col(u)) = x[u] * inv * at(s.keep_gain + col(u));
  }
  // everything the row needs is requested before the first meeting of the work-group
  T y[PER], past[PER], next[PER], looked[PER];           // past: of the average; looked: what the convolution sees of earlier inputs
  const int taps = s.conv.taps;
  const bool conv = SINGLE && s.conv.w;
  const int pos = conv ? r.pos[row] : 0;
  float* ring = conv ? s.ring + r.slot[row] * s.ring_elems : nullptr;
  float q = 0.0f;
#pragma unroll
  for (int u = 0; u < PER; u++) {
    const int c = col(u) < w ? col(u) : 0;
    y[u] = past[u] = next[u] = looked[u] = T{};
    if (s.y) {
      const float* p = s.y + row * s.parts * w + c;
      y[u] = at(p);
#pragma unroll 4
      for (int k = 1; k < s.parts; k++) y[u] += at(p + (int64_t)k * w);
    }
    if (s.kept && s.avg) {
      const float* k = s.kept + row * w + c;
#pragma unroll 4
      for (int j = 0; j < s.n_kept; j++) past[u] += at(k + j * s.kept_stride) * s.avg[j];
    }
    if (s.next) next[u] = at(s.next + c);
    if (conv)
      for (int j = 1; j < taps && j <= pos; j++) looked[u] += at(ring + (int64_t)((pos - j) % taps) * w + c) * at(s.conv.w + (int64_t)(taps - 1 - j) * w + c);
  }
  if (s.y) {
    T post[PER];
#pragma unroll
    for (int u = 0; u < PER; u++) { post[u] = at(s.post + (col(u) < w ? col(u) : 0)); if (col(u) < w) q += X::square(y[u]); }
    const float inv = 1.0f / sqrtf(group_total<THREADS>(q, red[0]) / (float)w + s.eps);
#pragma unroll
    for (int u = 0; u < PER; u++) x[u] += y[u] * inv * post[u];
  }
  if (s.kept) {
#pragma unroll
    for (int u = 0; u < PER; u++) {
      if (col(u) < w) *reinterpret_cast<T*>(s.kept + s.n_kept * s.kept_stride + row * w + col(u)) = x[u];
      if (s.avg) x[u] = past[u] + x[u] * s.avg[s.n_kept];
    }
  }
  if (s.y || a.e || s.kept) {
#pragma unroll
    for (int u = 0; u < PER; u++) if (col(u) < w) *reinterpret_cast<T*>(xr + col(u)) = x[u];
  }
  if (!s.next) return;
  q = 0.0f;
#pragma unroll
  for (int u = 0; u < PER; u++) if (col(u) < w) q += X::square(x[u]);
  const float inv = 1.0f / sqrtf(group_total<THREADS>(q, red[1]) / (float)w + s.eps);
  if (!SINGLE && s.conv.w) {
    if (tid == 0) s.inv[row] = inv;
    return;
  }
#pragma unroll
  for (int u = 0; u < PER; u++) {
    const int c = col(u);
    if (c >= w) continue;
    const T n = x[u] * inv * next[u];
    T h = n;
    if (conv) {
      h += n * at(s.conv.w + (int64_t)(taps - 1) * w + c) + looked[u];
      *reinterpret_cast<T*>(ring + (int64_t)(pos % taps) * w + c) = n;
    }
    X::template put<AT>(s.h, row * s.ldh + c, h);
  }
}

// h = n + conv(n) with n = x inv gain, eight rows a thread; the convolution slides over them (TAPS 0: any number, every row looks back)
constexpr int CONV_ROWS = 8;
template <typename AT, int V, int TAPS>
__global__ __launch_bounds__(256) void input_conv_kernel(const StreamStep s, const StepRows r)
{
  typedef Vec<V> X; typedef typename X::T T;
  constexpr int W = TAPS ? TAPS : 1;
  const int w = s.width, c = (blockIdx.y * 256 + threadIdx.x) * V, taps = TAPS ? TAPS : s.conv.taps;
  if (c >= w) return;
  auto at = [](const float* p) -> T { return *reinterpret_cast<const T*>(p); };
  const int r0 = blockIdx.x * CONV_ROWS, r1 = min(r0 + CONV_ROWS, r.n_rows);
  const T gain = at(s.next + c);
  T tap[W], hist[W];
#pragma unroll
  for (int j = 0; j < W; j++) tap[j] = at(s.conv.w + (int64_t)(TAPS ? j : taps - 1) * w + c);
  auto input = [&](int row, int j, int back, int pos) -> T {     // n of j tokens before the row's
    if (j <= back) return at(s.x + (int64_t)(row - j) * w + c) * s.inv[row - j] * gain;
    if (j <= pos) return at(s.ring + r.slot[row] * s.ring_elems + (int64_t)((pos - j) % taps) * w + c);
    return T{};
  };
  for (int row = r0; row < r1; row++) {
    const int pos = r.pos[row], back = row - r.first[row];
    const T n = at(s.x + (int64_t)row * w + c) * s.inv[row] * gain;
    T h = n + n * tap[W - 1];
    if constexpr (TAPS > 0) {
      if (row == r0 || back == 0) {
#pragma unroll
        for (int j = 1; j < TAPS; j++) hist[j] = input(row, j, back, pos);
      }
#pragma unroll
      for (int j = 1; j < TAPS; j++) h += hist[j] * tap[TAPS - 1 - j];
#pragma unroll
      for (int j = TAPS - 1; j > 1; j--) hist[j] = hist[j - 1];
      if (TAPS > 1) hist[1] = n;
    } else
      for (int j = 1; j < taps && j <= pos; j++) h += input(row, j, back, pos) * at(s.conv.w + (int64_t)(taps - 1 - j) * w + c);
    X::template put<AT>(s.h, row * s.ldh + c, h);
  }
}

template <typename AT, int V, int PER, int THREADS>
static void run_stream(const StreamArg& a, const StepRows& r, bool single)
{
  if (single) hipLaunchKernelGGL((stream_kernel<AT, V, PER, THREADS, true>), dim3(r.n_rows), dim3(THREADS), 0, ctx().stream, a, r);
  else hipLaunchKernelGGL((stream_kernel<AT, V, PER, THREADS, false>), dim3(r.n_rows), dim3(THREADS), 0, ctx().stream, a, r);
}
template <typename AT> static int run_stream_t(const StreamStep& s, const StepRows& r, bool single)
{
  const StreamArg a{s, s.embed ? (const uint16_t*)s.embed->data : nullptr, s.embed ? (int)s.embed->ld : 0};
  const int w = s.width;
  const bool wide = single || r.n_rows <= 64;            // few rows: a work-group as large as possible
  if (w % 4 == 0) {
    if (wide && w <= 4096) run_stream<AT, 4, 1, 1024>(a, r, single);
    else if (w <= 1024) run_stream<AT, 4, 1, 256>(a, r, single);
    else if (w <= 2048) run_stream<AT, 4, 2, 256>(a, r, single);
    else if (w <= 4096) run_stream<AT, 4, 4, 256>(a, r, single);
    else run_stream<AT, 4, 4, 1024>(a, r, single);
  } else if (w <= 1024) run_stream<AT, 1, 4, 256>(a, r, single);
  else run_stream<AT, 1, 16, 1024>(a, r, single);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int launch_stream(const StreamStep& s, int act_t, const StepRows& r, bool single)
{
  CAI_REQUIRE(s.width >= 1 && s.width <= 16384, "stream: rows of %d values", s.width);
  CAI_REQUIRE(!s.conv.w || (s.conv.taps >= 1 && s.ring && (single || s.inv)), "stream: a convolution without its ring");
  return act_t == ACT_T_BF16 ? run_stream_t<bf16_t>(s, r, single) : run_stream_t<float>(s, r, single);
}

template <typename AT, int V> static void run_conv(const StreamStep& s, const StepRows& r)
{
  const dim3 grid((r.n_rows + CONV_ROWS - 1) / CONV_ROWS, (s.width + 256 * V - 1) / (256 * V));
#define CONV(T) hipLaunchKernelGGL((input_conv_kernel<AT, V, T>), grid, dim3(256), 0, ctx().stream, s, r)
  switch (s.conv.taps) { case 2: CONV(2); break; case 3: CONV(3); break; case 4: CONV(4); break; default: CONV(0); }
#undef CONV
}
int launch_input_conv(const StreamStep& s, int act_t, const StepRows& r)
{
  CAI_REQUIRE(s.conv.w && s.conv.taps >= 1 && s.next && s.inv && s.ring && s.h, "input convolution: without operands");
  if (act_t == ACT_T_BF16) { if (s.width % 4 == 0) run_conv<bf16_t, 4>(s, r); else run_conv<bf16_t, 1>(s, r); }
  else { if (s.width % 4 == 0) run_conv<float, 4>(s, r); else run_conv<float, 1>(s, r); }
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

}  // namespace cai
