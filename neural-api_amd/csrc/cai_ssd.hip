// State-space duality (Mamba-2) mixers: prompt kernels (convolution and step sizes, scores, the walk over chunks, the gated group
// norm) and a decode kernel.
//
// Per head a float state S [state][vdim] (rows padded to four columns, the padding stays zero); one token does
//     S <- exp(rate dt) S + dt B x^T,   y = S^T C + D x,   dt = softplus(. + bias),   rate = -exp(A_log),
// with B and C shared by the heads of a group, and x, B and C behind one causal convolution and silu.  Everything that touches the
// state is 32-bit, the products of prompts run on the float matrix cores.
#include "cai_recurrent.hpp"

#include <algorithm>

namespace cai {

// ------------------------------------------------------------------------------------------
// prompt pass 1: x, B, C behind their convolution, step sizes.  A wave owns 256 channels (or the step sizes, or the zeros of the
// padding) over eight consecutive rows; the convolution slides over them, so each input is fetched once (TAPS 0: any number, every
// row looks back).
// ------------------------------------------------------------------------------------------
constexpr int SSD_PREP_ROWS = 8;

template <int TAPS>
__global__ __launch_bounds__(256) void ssd_prep_kernel(const SsdDims d, const SsdIn in, const SsdW w, const float* hist, const int64_t h_elems, const StepRows r, const SsdBuf b)
{
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r0 = blockIdx.x * SSD_PREP_ROWS, r1 = min(r0 + SSD_PREP_ROWS, r.n_rows);
  const int C = d.channels(), inner = d.inner(), gn = d.groups * d.state, np = d.np(), xp = d.xp();
  const int units = (C + 255) / 256;
  int unit = blockIdx.y * 4 + wave;
  if (unit < units) {
    const int c0 = unit * 256, n = min(256, C - c0);
    float *dst[4], bias[4]; int64_t step[4];             // where a channel goes, and its row stride
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int c = c0 + min(lane + 64 * i, n - 1);
      bias[i] = w.conv_b[c];
      if (c < inner) { dst[i] = b.x + c / d.vdim * xp + c % d.vdim; step[i] = d.heads * xp; }
      else {
        const int e = c < inner + gn ? c - inner : c - inner - gn;
        dst[i] = (c < inner + gn ? b.B : b.C) + e / d.state * np + e % d.state; step[i] = d.groups * np;
      }
    }
    ConvWindow<TAPS ? TAPS : 2> cw;
    if (TAPS) cw.taps(w.conv, c0, lane, n);
    for (int row = r0; row < r1; row++) {
      const int pos = r.pos[row], back = row - r.first[row];
      const float* ring = hist + r.slot[row] * h_elems;
      const float* p = in.proj + row * in.ldp + in.ox;
      if (TAPS && (row == r0 || back == 0)) cw.history(p, in.ldp, back, pos, ring, C, 0, c0, lane, n);
      float x[4];
#pragma unroll
      for (int i = 0; i < 4; i++) x[i] = p[c0 + min(lane + 64 * i, n - 1)];
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int c = lane + 64 * i;
        if (TAPS) x[i] = cw.step(i, x[i], bias[i]);
        else if (c < n) x[i] = conv_silu(p, in.ldp, back, pos, ring, C, 0, w.conv, d.taps, c0 + c, bias[i]);
        if (c < n) dst[i][row * step[i]] = x[i];
      }
    }
    return;
  }
  if (unit == units) {
    for (int row = r0; row < r1; row++)
      for (int h = lane; h < d.heads; h += 64) b.dt[(int64_t)row * d.heads + h] = softplus_f(in.proj[row * in.ldp + in.odt + h] + w.dt_bias[h]);
    return;
  }
  if (unit == units + 1) {
    const int px = xp - d.vdim, pn = np - d.state;
    for (int row = r0; row < r1; row++) {
      for (int e = lane; e < d.heads * px; e += 64) b.x[((int64_t)row * d.heads + e / px) * xp + d.vdim + e % px] = 0.0f;
      for (int e = lane; e < d.groups * pn; e += 64) {
        const int64_t at = ((int64_t)row * d.groups + e / pn) * np + d.state + e % pn;
        b.B[at] = 0.0f; b.C[at] = 0.0f;
      }
    }
  }
}

// ------------------------------------------------------------------------------------------
// prompt pass 2: C B^T of a chunk and group, on and below the diagonal (a wave per 16 rows).  Rows past the portion's end are other
// rows of the buffers: their scores are never used.
// ------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void ssd_scores_kernel(const SsdDims d, const StepRows r, const SsdBuf b, const int32_t* chunks)
{
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), fr = lane & 15, fg = lane >> 4;
  const int32_t* en = r.ent + 4 * chunks[2 * blockIdx.x];
  const int t0 = chunks[2 * blockIdx.x + 1], nt = min(SSD_CHUNK, en[2] - t0), g = blockIdx.y, np = d.np();
  if (wave * 16 >= nt) return;
  const int64_t row0 = en[1] + t0, ld = (int64_t)d.groups * np;
  const float* cp = b.C + (row0 + min(wave * 16 + fr, nt - 1)) * ld + g * np + fg * 4;
  const float* bp[4];
  f32x4 acc[4];
#pragma unroll
  for (int t = 0; t < 4; t++) { bp[t] = b.B + (row0 + min(t * 16 + fr, nt - 1)) * ld + g * np + fg * 4; acc[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f}; }
  for (int k = 0; k < np; k += 16) {
    const f32x4 c = *reinterpret_cast<const f32x4*>(cp + k);
#pragma unroll
    for (int t = 0; t < 4; t++) {
      if (t > wave) continue;
      const f32x4 x = *reinterpret_cast<const f32x4*>(bp[t] + k);
#pragma unroll
      for (int i = 0; i < 4; i++) acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(c[i], x[i], acc[t], 0, 0, 0);
    }
  }
  float* o = b.cb + ((int64_t)blockIdx.x * d.groups + g) * SSD_CHUNK * SSD_CHUNK;
#pragma unroll
  for (int t = 0; t < 4; t++)
#pragma unroll
    for (int i = 0; i < 4; i++) if (t <= wave) o[(wave * 16 + fg * 4 + i) * SSD_CHUNK + t * 16 + fr] = acc[t][i];
}

// ------------------------------------------------------------------------------------------
// prompt pass 3: the walk, one work-group per (16 columns of a head, entry).  With L_t the sum of rate dt over the chunk's tokens up
// to t and S the state before the chunk,
//     y_t = exp(L_t) S^T C_t + sum_{s<=t} (C_t . B_s) exp(L_t - L_s) dt_s x_s + D x_t,
//     S <- exp(L_last) S + sum_s B_s exp(L_last - L_s) dt_s x_s^T.
// Wave w makes the outputs of the chunk's tokens 16 w .. 16 w + 15 and holds the state rows of tiles w + 4 j as matrix-core result
// registers, which pass to the other waves as operands through LDS (two copies, one barrier a chunk).  L is kept in double
// precision, so that differences of large sums cost no accuracy.
// ------------------------------------------------------------------------------------------
template <int TPW>
__global__ __launch_bounds__(256) void ssd_walk_kernel(const SsdDims d, const SsdW w, float* state, const int64_t s_elems, const StepRows r, const SsdBuf b, const int32_t* chunk0)
{
  __shared__ f32x4 sS[2][TPW * 4][64];
  __shared__ double sL[4][SSD_CHUNK];
  __shared__ float sdt[4][SSD_CHUNK];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), fr = lane & 15, fg = lane >> 4;
  const int slices = (d.vdim + 15) / 16;
  // consecutive work-groups go to different XCDs; with heads in whole eights a head's slices stay on one
  const int h = d.heads % 8 == 0 ? (blockIdx.x & 7) + 8 * ((blockIdx.x >> 3) / slices) : blockIdx.x / slices;
  const int col = (d.heads % 8 == 0 ? (blockIdx.x >> 3) % slices : blockIdx.x % slices) * 16 + fr;
  const int32_t* en = r.ent + 4 * blockIdx.y;
  const int slot = en[0], row0 = en[1], n = en[2], pos0 = en[3], ch0 = chunk0[blockIdx.y];
  const int g = h / (d.heads / d.groups), np = d.np(), xp = d.xp(), dvp = d.vdim_p(), tiles = np / 16;
  const int64_t ldb = (int64_t)d.groups * np, ldx = (int64_t)d.heads * xp;
  const float rate = w.rate[h], skip = w.D[h];
  float* Sg = state + slot * s_elems + (int64_t)h * d.state * dvp;
  f32x4 S[TPW];
#pragma unroll
  for (int j = 0; j < TPW; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int rr = (wave + 4 * j) * 16 + fg * 4 + i;
      S[j][i] = pos0 > 0 && rr < d.state && col < d.vdim ? Sg[(int64_t)rr * dvp + col] : 0.0f;
    }
  for (int c = 0; c * SSD_CHUNK < n; c++) {
    const int nt = min(SSD_CHUNK, n - c * SSD_CHUNK);
    const int64_t rr = row0 + c * SSD_CHUNK;
    // requests of the chunk; rows past the end repeat the last one (their step size is zero)
    const bool out = wave * 16 < nt;
    f32x4 cf[TPW * 4], cbf[4];
    float x[4][4], bf[TPW][4][4];
    const float dtv = b.dt[(rr + min(lane, nt - 1)) * d.heads + h];
#pragma unroll
    for (int t = 0; t < 4; t++)
#pragma unroll
      for (int i = 0; i < 4; i++) x[t][i] = b.x[(rr + min(t * 16 + fg * 4 + i, nt - 1)) * ldx + h * xp + col];
    if (out) {
      const float* cp = b.C + (rr + min(wave * 16 + fr, nt - 1)) * ldb + g * np + fg * 4;
#pragma unroll
      for (int k = 0; k < TPW * 4; k++) if (k < tiles) cf[k] = *reinterpret_cast<const f32x4*>(cp + k * 16);
      const float* cb = b.cb + (((int64_t)(ch0 + c) * d.groups + g) * SSD_CHUNK + wave * 16 + fr) * SSD_CHUNK + fg * 4;
#pragma unroll
      for (int t = 0; t < 4; t++) if (t <= wave) cbf[t] = *reinterpret_cast<const f32x4*>(cb + t * 16);
    }
#pragma unroll
    for (int j = 0; j < TPW; j++)
      if (wave + 4 * j < tiles)
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
          for (int i = 0; i < 4; i++) bf[j][t][i] = b.B[(rr + min(t * 16 + fg * 4 + i, nt - 1)) * ldb + g * np + (wave + 4 * j) * 16 + fr];
#pragma unroll
    for (int j = 0; j < TPW; j++) sS[c & 1][wave + 4 * j][lane] = S[j];
    // running sums of the logarithms of the decays, a token a lane
    double L = lane < nt ? (double)(rate * dtv) : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) { const double u = __shfl_up(L, o); if (lane >= o) L += u; }
    sL[wave][lane] = L; sdt[wave][lane] = lane < nt ? dtv : 0.0f;
    __syncthreads();
    const double last = sL[wave][SSD_CHUNK - 1];
    float xd[4][4];
#pragma unroll
    for (int t = 0; t < 4; t++)
#pragma unroll
      for (int i = 0; i < 4; i++) xd[t][i] = x[t][i] * sdt[wave][t * 16 + fg * 4 + i];
    if (out) {
      f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f}, y2 = y;
#pragma unroll
      for (int k = 0; k < TPW * 4; k++) {
        if (k >= tiles) continue;
        const f32x4 sf = sS[c & 1][k][lane];
#pragma unroll
        for (int i = 0; i < 4; i++) {
          if (k & 1) y2 = __builtin_amdgcn_mfma_f32_16x16x4f32(cf[k][i], sf[i], y2, 0, 0, 0);
          else y = __builtin_amdgcn_mfma_f32_16x16x4f32(cf[k][i], sf[i], y, 0, 0, 0);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; i++) y[i] = (y[i] + y2[i]) * expf((float)sL[wave][wave * 16 + fg * 4 + i]);
      const double Lt = sL[wave][wave * 16 + fr];
#pragma unroll
      for (int t = 0; t < 4; t++) {
        if (t > wave) continue;
#pragma unroll
        for (int i = 0; i < 4; i++) {
          const int s = t * 16 + fg * 4 + i;
          const float gv = s <= wave * 16 + fr ? cbf[t][i] * expf((float)(Lt - sL[wave][s])) : 0.0f;
          y = __builtin_amdgcn_mfma_f32_16x16x4f32(gv, xd[t][i], y, 0, 0, 0);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int t = wave * 16 + fg * 4 + i;
        float own = x[0][i];
#pragma unroll
        for (int q = 1; q < 4; q++) own = q == wave ? x[q][i] : own;
        if (t < nt && col < d.vdim) b.y[(rr + t) * d.inner() + h * d.vdim + col] = fmaf(skip, own, y[i]);
      }
    }
    const float all = expf((float)last);
#pragma unroll
    for (int j = 0; j < TPW; j++) S[j] *= all;
#pragma unroll
    for (int t = 0; t < 4; t++) {
      if (t * 16 >= nt) continue;
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const float xs = xd[t][i] * expf((float)(last - sL[wave][t * 16 + fg * 4 + i]));
#pragma unroll
        for (int j = 0; j < TPW; j++) if (wave + 4 * j < tiles) S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(bf[j][t][i], xs, S[j], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int j = 0; j < TPW; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int rr = (wave + 4 * j) * 16 + fg * 4 + i;
      if (rr < d.state && col < dvp) Sg[(int64_t)rr * dvp + col] = S[j][i];
    }
}

// ------------------------------------------------------------------------------------------
// decode: one token of each entry, one work-group per (head, row): convolutions, step size, state update, read-out.  The state is
// requested first and sits in registers while the rest is made.
// ------------------------------------------------------------------------------------------
template <int RPT>
__global__ __launch_bounds__(512) void ssd_single_kernel(const SsdDims d, const SsdIn in, const SsdW w, float* state, const int64_t s_elems, float* hist, const int64_t h_elems, const StepRows r, float* y, const int ct_log)
{
  __shared__ float sx[256], sB[256], sC[256];
  __shared__ f32x4 red[8][32];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int pos = r.pos[row], slot = r.slot[row], hg = d.heads / d.groups, g = h / hg, C = d.channels(), inner = d.inner(), dvp = d.vdim_p();
  // a thread holds four consecutive columns of RPT rows; CT threads a row, RG rows side by side
  const int CT = 1 << ct_log, CP = CT * 4, RG = 512 >> ct_log, ct = tid & (CT - 1), rg = tid >> ct_log;
  float* Sg = state + slot * s_elems + (int64_t)h * d.state * dvp;
  f32x4 S[RPT];
  auto load_state = [&](int c0) {
#pragma unroll
    for (int j = 0; j < RPT; j++) {
      const int rr = rg + j * RG;
      S[j] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
      if (pos > 0 && rr < d.state && c0 + ct * 4 < dvp) S[j] = *reinterpret_cast<const f32x4*>(Sg + (unsigned)(rr * dvp + c0 + ct * 4));
    }
  };
  load_state(0);
  const float* p = in.proj + row * in.ldp;
  float* ring = hist + slot * h_elems;
  float* ring_now = ring + (int64_t)(pos % d.taps) * C;
  for (int e = tid; e < d.vdim + 2 * d.state; e += 512) {
    const int k = e - d.vdim;
    const int c = k < 0 ? h * d.vdim + e : k < d.state ? inner + g * d.state + k : inner + d.groups * d.state + g * d.state + k - d.state;
    const float v = conv_silu(p + in.ox, in.ldp, 0, pos, ring, C, 0, w.conv, d.taps, c, w.conv_b[c]);
    if (k < 0) sx[e] = v; else if (k < d.state) sB[k] = v; else sC[k - d.state] = v;
    if (k < 0 || h % hg == 0) ring_now[c] = p[in.ox + c];
  }
  const float dt = softplus_f(p[in.odt + h] + w.dt_bias[h]), decay = expf(w.rate[h] * dt), skip = w.D[h];
  __syncthreads();
  for (int c0 = 0; c0 < d.vdim; c0 += CP) {
    if (c0) load_state(c0);
    f32x4 x, o = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int i = 0; i < 4; i++) x[i] = c0 + ct * 4 + i < d.vdim ? sx[c0 + ct * 4 + i] * dt : 0.0f;
#pragma unroll
    for (int j = 0; j < RPT; j++) {
      const int rr = rg + j * RG;
      if (rr >= d.state || c0 + ct * 4 >= dvp) continue;
      const float bv = sB[rr], cv = sC[rr];
#pragma unroll
      for (int i = 0; i < 4; i++) { S[j][i] = fmaf(bv, x[i], S[j][i] * decay); o[i] = fmaf(S[j][i], cv, o[i]); }
      *reinterpret_cast<f32x4*>(Sg + (unsigned)(rr * dvp + c0 + ct * 4)) = S[j];
    }
    for (int m = CT; m < 64; m <<= 1)
#pragma unroll
      for (int i = 0; i < 4; i++) o[i] += __shfl_xor(o[i], m);
    if (c0) __syncthreads();
    if (lane < CT) red[wave][ct] = o;
    __syncthreads();
    if (tid < CP && c0 + tid < d.vdim) {
      float s = 0.0f;
#pragma unroll
      for (int i = 0; i < 8; i++) s += reinterpret_cast<const float*>(red[i])[tid];
      y[(int64_t)row * inner + h * d.vdim + c0 + tid] = fmaf(skip, sx[c0 + tid], s);
    }
  }
}

// ------------------------------------------------------------------------------------------
// gate, then RMS norm of each of norm_groups equal parts, gain.  Up to sixteen values a thread stay in registers; wider parts are made
// again.  The first part's work-group of a portion's last rows also keeps their raw inputs (a decoded token's are kept already).
// ------------------------------------------------------------------------------------------
template <typename AT>
__global__ __launch_bounds__(512) void ssd_finish_kernel(const SsdDims d, const SsdIn in, const SsdW w, float* hist, const int64_t h_elems, const StepRows r, const float* y, const int single, AT* out, const int64_t ldo)
{
  __shared__ float part[8];
  const int64_t row = blockIdx.x;
  const int tid = threadIdx.x, inner = d.inner(), gw = inner / d.norm_groups, c0 = blockIdx.y * gw;
  const float *p = in.proj + row * in.ldp, *yr = y + row * inner + c0, *z = p + in.oz + c0;
  auto gated = [&](int c) -> float { const float v = z[c]; return yr[c] * (v * sigmoid_f(v)); };
  float u[16], s = 0.0f;
#pragma unroll
  for (int i = 0; i < 16; i++) { const int c = tid + i * 512; u[i] = 0.0f; if (c < gw) u[i] = gated(c); s = fmaf(u[i], u[i], s); }
  for (int c = tid + 16 * 512; c < gw; c += 512) { const float v = gated(c); s = fmaf(v, v, s); }
  s = wave_total(s);
  if ((tid & 63) == 0) part[tid >> 6] = s;
  __syncthreads();
  s = 0.0f;
#pragma unroll
  for (int i = 0; i < 8; i++) s += part[i];
  const float inv = 1.0f / sqrtf(s / (float)gw + d.eps);
#pragma unroll
  for (int i = 0; i < 16; i++) { const int c = tid + i * 512; if (c < gw) out[row * ldo + c0 + c] = (AT)(u[i] * inv * w.norm[c0 + c]); }
  for (int c = tid + 16 * 512; c < gw; c += 512) out[row * ldo + c0 + c] = (AT)(gated(c) * inv * w.norm[c0 + c]);
  if (!single && blockIdx.y == 0 && r.last[row] - row < d.taps) {
    const int C = d.channels();
    float* ring = hist + r.slot[row] * h_elems + (int64_t)(r.pos[row] % d.taps) * C;
    for (int c = tid; c < C; c += 512) ring[c] = p[in.ox + c];
  }
}

int ssd_prep(const SsdDims& d, const SsdIn& in, const SsdW& w, const SeqPool::StateRun& st, const StepRows& r, const SsdBuf& b)
{
  const bool pads = d.np() != d.state || d.xp() != d.vdim;
  const int units = (d.channels() + 255) / 256 + (pads ? 2 : 1);
  const dim3 grid((r.n_rows + SSD_PREP_ROWS - 1) / SSD_PREP_ROWS, (units + 3) / 4);
#define PREP(T) hipLaunchKernelGGL(ssd_prep_kernel<T>, grid, dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b)
  if (d.taps == 2) PREP(2); else if (d.taps == 3) PREP(3); else if (d.taps == 4) PREP(4); else PREP(0);
#undef PREP
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int ssd_walk(const SsdDims& d, const SsdW& w, const SeqPool::StateRun& st, const StepRows& r, const SsdBuf& b, const int32_t* chunks, int n_chunks, const int32_t* chunk0)
{
  hipLaunchKernelGGL(ssd_scores_kernel, dim3(n_chunks, d.groups), dim3(256), 0, ctx().stream, d, r, b, chunks);
  const dim3 grid((d.vdim + 15) / 16 * d.heads, r.n_ent);
#define WALK(N) hipLaunchKernelGGL(ssd_walk_kernel<N>, grid, dim3(256), 0, ctx().stream, d, w, st.S, st.s_elems, r, b, chunk0)
  if (d.state <= 64) WALK(1); else if (d.state <= 128) WALK(2); else WALK(4);
#undef WALK
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int ssd_single(const SsdDims& d, const SsdIn& in, const SsdW& w, const SeqPool::StateRun& st, const StepRows& r, const SsdBuf& b)
{
  const int ct_log = d.vdim > 64 ? 5 : d.vdim > 32 ? 4 : 3, rgs = 512 >> ct_log, rpt = (d.state + rgs - 1) / rgs;
#define SINGLE(N) hipLaunchKernelGGL(ssd_single_kernel<N>, dim3(d.heads, r.n_rows), dim3(512), 0, ctx().stream, d, in, w, st.S, st.s_elems, st.hist, st.h_elems, r, b.y, ct_log)
  if (rpt <= 2) SINGLE(2); else if (rpt <= 4) SINGLE(4); else if (rpt <= 8) SINGLE(8); else SINGLE(16);
#undef SINGLE
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int ssd_finish(const SsdDims& d, const SsdIn& in, const SsdW& w, const SeqPool::StateRun& st, const StepRows& r, const SsdBuf& b, bool single, int act_t, void* out, int64_t ldo)
{
  const dim3 grid(r.n_rows, d.norm_groups);
  if (act_t == ACT_T_BF16) hipLaunchKernelGGL(ssd_finish_kernel<bf16_t>, grid, dim3(512), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b.y, single ? 1 : 0, (bf16_t*)out, ldo);
  else hipLaunchKernelGGL(ssd_finish_kernel<float>, grid, dim3(512), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b.y, single ? 1 : 0, (float*)out, ldo);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

}  // namespace cai
