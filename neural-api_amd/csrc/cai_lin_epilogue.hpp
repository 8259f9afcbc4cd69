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

__device__ __forceinline__ float lin_act(float v, int act)
{
  if (act == LIN_RELU_SQUARED) { v = fmaxf(v, 0.0f); return v * v; }
  return act_apply(v, act);
}
// factor of a sublayer's result before it joins the stream
__device__ __forceinline__ float join_factor(const LinEpi& e, int n, int64_t t)
{
  float f = e.mult ? e.mult[n] : 1.0f;
  if (e.gate) f /= 1.0f + expf(-e.gate[t * e.ldg + n]);
  return f;
}

template <typename AT> __device__ __forceinline__ void put_act(void* p, int64_t i, float v)
{
  if constexpr (sizeof(AT) == 2) reinterpret_cast<uint16_t*>(p)[i] = bf16_bits(v);
  else reinterpret_cast<float*>(p)[i] = v;
}

// one finished sum of STORE / RESIDUAL / SPLIT
template <typename AT> __device__ __forceinline__ void epi_one(const LinEpi& e, int n, int t, float v)
{
  if (e.mode == EPI_STORE) {
    v *= e.scale;
    if (e.bias) v += e.bias[n];
    e.y[t * e.ldy + n] = lin_act(v, e.act);
  } else if (e.mode == EPI_SPLIT) {
    if (e.bias) v += e.bias[n];
    if (n < e.split) e.y[t * e.ldy + n] = v;
    else put_act<AT>(e.h, t * e.ldh + n - e.split, lin_act(v, e.act));
  } else {
    if (e.bias) v += e.bias[n];
    if (e.mult || e.gate) v *= join_factor(e, n, t);
    float x = (e.fresh ? 0.0f : e.y[t * e.ldy + n]) + dyt(e.post, v, n);
    if (e.add0) x += e.add0[t * e.ld0 + n];
    e.y[t * e.ldy + n] = x;
    if (e.h) put_act<AT>(e.h, t * e.ldh + n, dyt(e.next, x, n));
  }
}

}  // namespace cai
