// Device functions shared by the recurrent mixers: wave sums, soft-plus and sigmoid, causal convolutions with silu.
//
// A sequence's last `taps` raw inputs of every convolved channel are kept in a ring (entry position mod taps).  The ring has one
// entry more than a token looks back, so the entry the newest token takes is never one that the same step still reads.
#pragma once
#include "cai_layered.hpp"
#include "cai_gemv_common.hpp"

namespace cai {

__device__ __forceinline__ float wave_total(float v)   // the sum in every lane
{
  v = wave_sum(v);
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), 63));
}
__device__ __forceinline__ float sigmoid_f(float z)
{
  if (z >= 0.0f) return 1.0f / (1.0f + expf(-z));
  const float s = expf(z); return s / (1.0f + s);
}
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
template <int CTRL> __device__ __forceinline__ float dpp_add(float v)
{
  return v + __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float row16_total(float v)  // the sum over the lane's row of 16, in every lane of it (row rotations)
{
  v = dpp_add<0x128>(v); v = dpp_add<0x124>(v); v = dpp_add<0x122>(v); return dpp_add<0x121>(v);
}

// convolution + silu of channel c (column oc + c of the raw projections, ring channel hc + c) for a row `back` rows into its entry
__device__ __forceinline__ float conv_silu(const float* cur, int64_t ldp, int back, int pos, const float* ring, int channels, int hc, const float* w, int taps, int c, float bias = 0.0f)
{
  float s = fmaf(w[c * taps + taps - 1], cur[c], bias);
  for (int j = 1; j < taps; j++) {
    float x = 0.0f;
    if (j <= back) x = cur[c - (int64_t)j * ldp];
    else if (j <= pos) x = ring[(int64_t)((pos - j) % taps) * channels + hc + c];
    s = fmaf(w[c * taps + taps - 1 - j], x, s);
  }
  return s * sigmoid_f(s);
}

template <int TAPS>
struct ConvWindow {                        // four channels of a lane: c = lane + 64 i
  float w[4][TAPS], h[4][TAPS - 1];        // taps, the inputs before the current one (h[0] the latest)
  __device__ __forceinline__ void taps(const float* cw, int c0, int lane, int n)
  {
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int k = 0; k < TAPS; k++) { const int c = lane + 64 * i; w[i][k] = c < n ? cw[(c0 + c) * TAPS + k] : 0.0f; }
  }
  __device__ __forceinline__ void history(const float* cur, int64_t ldp, int back, int pos, const float* ring, int channels, int hc, int c0, int lane, int n)
  {
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int j = 1; j < TAPS; j++) {
        const int c = lane + 64 * i;
        h[i][j - 1] = 0.0f;
        if (c < n) {
          if (j <= back) h[i][j - 1] = cur[c0 + c - (int64_t)j * ldp];
          else if (j <= pos) h[i][j - 1] = ring[(int64_t)((pos - j) % TAPS) * channels + hc + c0 + c];
        }
      }
  }
  __device__ __forceinline__ float step(int i, float x, float bias = 0.0f)
  {
    float s = fmaf(w[i][TAPS - 1], x, bias);
#pragma unroll
    for (int j = 1; j < TAPS; j++) s = fmaf(w[i][TAPS - 1 - j], h[i][j - 1], s);
#pragma unroll
    for (int j = TAPS - 2; j > 0; j--) h[i][j] = h[i][j - 1];
    h[i][0] = x;
    return s * sigmoid_f(s);
  }
};

}  // namespace cai
