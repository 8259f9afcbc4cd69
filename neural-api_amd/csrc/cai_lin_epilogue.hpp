// What a product over bfloat16 weights does with its finished 32-bit sums.
#pragma once
#include "cai_layered.hpp"
#include "cai_gemv_common.hpp"

namespace cai {

__device__ __forceinline__ float glu_pair(int kind, float limit, float g, float u)
{
  if (kind == GLU_RELU) return fmaxf(g, 0.0f) * u;
  if (kind == GLU_SILU) return silu_mul(u, g);
  if (kind == GLU_GELU_TANH) return 0.5f * g * (1.0f + tanhf(0.79788456080286535588f * fmaf(0.044715f * g * g, g, g))) * u;
  g = fminf(g, limit); u = fminf(fmaxf(u, -limit), limit);
  return g / (1.0f + expf(-1.702f * g)) * (u + 1.0f);
}

__device__ __forceinline__ float lin_act(float v, int act, float limit)
{
  if (act == LIN_SOFT_CAP) return limit * tanhf(v / limit);
  if (act == LIN_RELU_SQUARED) { v = fmaxf(v, 0.0f); return v * v; }
  return act_apply(v, act);
}
// four of them; the kinds the products of a layer have cost no more than a branch, and one loop holds the others (64 copies of those in a
// kernel's epilogue, each visited once, would wait for instructions longer than the product takes)
__device__ __forceinline__ f32x4 lin_act_four(f32x4 v, int act, float limit)
{
  if (act == CAI_ACT_NONE) return v;
  if (act == LIN_RELU_SQUARED) {
#pragma unroll
    for (int q = 0; q < 4; q++) { const float p = fmaxf(v[q], 0.0f); v[q] = p * p; }
    return v;
  }
#pragma unroll 1
  for (int q = 0; q < 4; q++) v = f32x4{v[1], v[2], v[3], lin_act(v[0], act, limit)};
  return v;
}
// factor of a sublayer's result before it joins the stream
__device__ __forceinline__ float join_factor(const LinEpi& e, int n, int64_t t)
{
  return e.mult[n] / (1.0f + expf(-e.gate[t * e.ldg + n]));
}

// two finished sums of the same output, both joined
__device__ __forceinline__ void join_two(const LinEpi& a, float va, const LinEpi& b, float vb, int n, int64_t t)
{
  if (a.bias) va += a.bias[n];
  if (b.bias) vb += b.bias[n];
  a.y[t * a.ldy + n] += va * join_factor(a, n, t) + vb * join_factor(b, n, t);
}

template <typename AT> __device__ __forceinline__ void put_act(void* p, int64_t i, float v)
{
  if constexpr (sizeof(AT) == 2) reinterpret_cast<uint16_t*>(p)[i] = bf16_bits(v);
  else reinterpret_cast<float*>(p)[i] = v;
}

// one finished sum of any mode but GLU
template <typename AT, int MODE> __device__ __forceinline__ void epi_as(const LinEpi& e, int n, int64_t t, float v)
{
  if constexpr (MODE == EPI_STORE) v *= e.scale;
  if (e.bias) v += e.bias[n];
  float* y = e.y + t * e.ldy + n;
  if constexpr (MODE == EPI_STORE) *y = lin_act(v, e.act, e.limit);
  else if constexpr (MODE == EPI_SPLIT) {
    if (n < e.split) *y = v;
    else put_act<AT>(e.h, t * e.ldh + n - e.split, lin_act(v, e.act, e.limit));
  } else if constexpr (MODE == EPI_JOIN) *y += v * join_factor(e, n, t);
  else {
    float x = (e.fresh ? 0.0f : *y) + dyt(e.post, v, n);
    if (e.add0) x += e.add0[t * e.ld0 + n];
    *y = x;
    if (e.h) put_act<AT>(e.h, t * e.ldh + n, dyt(e.next, x, n));
  }
}
template <typename AT> __device__ __forceinline__ void epi_one(const LinEpi& e, int n, int64_t t, float v)
{
  if (e.mode == EPI_STORE) epi_as<AT, EPI_STORE>(e, n, t, v);
  else if (e.mode == EPI_SPLIT) epi_as<AT, EPI_SPLIT>(e, n, t, v);
  else if (e.mode == EPI_JOIN) epi_as<AT, EPI_JOIN>(e, n, t, v);
  else epi_as<AT, EPI_RESIDUAL>(e, n, t, v);
}

// four consecutive ones, every stride and `split` a multiple of four
template <typename AT> __device__ __forceinline__ void put_four(void* p, int64_t i, f32x4 v)
{
  if constexpr (sizeof(AT) == 2)
    *reinterpret_cast<uint2*>(reinterpret_cast<uint16_t*>(p) + i) = make_uint2(bf16_bits(v[0]) | (uint32_t)bf16_bits(v[1]) << 16, bf16_bits(v[2]) | (uint32_t)bf16_bits(v[3]) << 16);
  else *reinterpret_cast<f32x4*>(reinterpret_cast<float*>(p) + i) = v;
}
template <typename AT, int MODE> __device__ __forceinline__ void epi_four(const LinEpi& e, int n, int64_t t, f32x4 v)
{
  if constexpr (MODE == EPI_STORE) v *= e.scale;
  if (e.bias) v += f32x4{e.bias[n], e.bias[n + 1], e.bias[n + 2], e.bias[n + 3]};
  f32x4* yp = reinterpret_cast<f32x4*>(e.y + t * e.ldy + n);
  if constexpr (MODE == EPI_STORE) {
    *yp = lin_act_four(v, e.act, e.limit);
  } else if constexpr (MODE == EPI_SPLIT) {
    if (n < e.split) { *yp = v; return; }
    put_four<AT>(e.h, t * e.ldh + n - e.split, lin_act_four(v, e.act, e.limit));
  } else if constexpr (MODE == EPI_JOIN) {
    const f32x4 g = *reinterpret_cast<const f32x4*>(e.gate + t * e.ldg + n);
    f32x4 x = *yp;
#pragma unroll
    for (int q = 0; q < 4; q++) x[q] += v[q] * (e.mult[n + q] / (1.0f + expf(-g[q])));
    *yp = x;
  } else {
    f32x4 x = {0.0f, 0.0f, 0.0f, 0.0f};
    if (!e.fresh) x = *yp;
#pragma unroll
    for (int q = 0; q < 4; q++) x[q] += dyt(e.post, v[q], n + q);
    if (e.add0) x += *reinterpret_cast<const f32x4*>(e.add0 + t * e.ld0 + n);
    *yp = x;
    if (e.h) {
#pragma unroll
      for (int q = 0; q < 4; q++) v[q] = dyt(e.next, x[q], n + q);
      put_four<AT>(e.h, t * e.ldh + n, v);
    }
  }
}

}  // namespace cai
