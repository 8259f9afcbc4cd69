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

template <typename AT> __device__ __forceinline__ void put_act(void* p, int64_t i, float v)
{
  if constexpr (sizeof(AT) == 2) reinterpret_cast<uint16_t*>(p)[i] = bf16_bits(v);
  else reinterpret_cast<float*>(p)[i] = v;
}

// one finished sum of STORE / RESIDUAL
template <typename AT> __device__ __forceinline__ void epi_one(const LinEpi& e, int n, int t, float v)
{
  if (e.mode == EPI_STORE) {
    if (e.bias) v += e.bias[n];
    e.y[t * e.ldy + n] = act_apply(v, e.act);
  } else {
    if (e.bias) v += e.bias[n];
    float x = (e.fresh ? 0.0f : e.y[t * e.ldy + n]) + dyt(e.post, v, n);
    if (e.add0) x += e.add0[t * e.ld0 + n];
    e.y[t * e.ldy + n] = x;
    if (e.h) put_act<AT>(e.h, t * e.ldh + n, dyt(e.next, x, n));
  }
}

}  // namespace cai
