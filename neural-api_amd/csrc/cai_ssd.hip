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
// prompt pass 2, everything of a chunk of 64 tokens that does not need the state.  With L_t the sum of rate dt over the chunk's tokens
// up to t and E_i its value at the end of the i-th 16 tokens (E_-1 = 0):
//   blockIdx.y < groups: C B^T of the group, on and below the diagonal, a wave per 16 x 16 tile;
//   the next `groups`: B of the group with the tokens along the rows (zero past the portion's end);
//   above: a wave per head leaves SSD_FACTORS floats,  u_s = dt_s exp(E_tile(s) - L_s),  dt_s,  l_t = L_t - E_tile(t)-1,  a_t = exp(l_t),
//   and the decays exp(E_i - E_i-1) of the four tiles.
// Every exponent is a sum within 16 tokens, made from double precision sums; longer decays are products of these, so strong decay
// costs no accuracy.  Tokens past the portion's end have step size zero.
// ------------------------------------------------------------------------------------------
constexpr int SCORE_WAVES = 10;
__global__ __launch_bounds__(64 * SCORE_WAVES) void ssd_chunk_kernel(const SsdDims d, const StepRows r, const SsdW w, const SsdBuf b, const int32_t* chunks)
{
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), fr = lane & 15, fg = lane >> 4;
  const int32_t* en = r.ent + 4 * chunks[2 * blockIdx.x];
  const int t0 = chunks[2 * blockIdx.x + 1], nt = min(SSD_CHUNK, en[2] - t0), np = d.np();
  const int64_t row0 = en[1] + t0;
  const int64_t ld = (int64_t)d.groups * np;
  if ((int)blockIdx.y >= d.groups && (int)blockIdx.y < 2 * d.groups) {
    const int g = blockIdx.y - d.groups;
    float* o = b.bt + ((int64_t)blockIdx.x * d.groups + g) * np * SSD_CHUNK;
    for (int n = wave; n < np; n += SCORE_WAVES) o[n * SSD_CHUNK + lane] = lane < nt ? b.B[(row0 + lane) * ld + g * np + n] : 0.0f;
    return;
  }
  if ((int)blockIdx.y >= 2 * d.groups) {
    const int h = (blockIdx.y - 2 * d.groups) * SCORE_WAVES + wave;
    if (h >= d.heads) return;
    const float dt = lane < nt ? b.dt[(row0 + lane) * d.heads + h] : 0.0f;
    double L = (double)(w.rate[h] * dt);
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) { const double u = __shfl_up(L, o); if (lane >= o) L += u; }
    const double end = __shfl(L, lane | 15), before = __shfl(L, max((lane & 48) - 1, 0));     // (every lane takes part)
    const float l = (float)(L - (lane < 16 ? 0.0 : before));
    float* f = b.fac + ((int64_t)blockIdx.x * d.heads + h) * SSD_FACTORS;
    f[lane] = dt * expf((float)(end - L)); f[64 + lane] = dt; f[128 + lane] = l; f[192 + lane] = expf(l);
    if (fr == 15) f[256 + fg] = expf(l);
    return;
  }
  const int g = blockIdx.y, tr = wave < 1 ? 0 : wave < 3 ? 1 : wave < 6 ? 2 : 3, tc = wave - tr * (tr + 1) / 2;
  if (tr * 16 >= nt) return;
  const float* cp = b.C + (row0 + min(tr * 16 + fr, nt - 1)) * ld + g * np + fg * 4;
  const float* bp = b.B + (row0 + min(tc * 16 + fr, nt - 1)) * ld + g * np + fg * 4;
  f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
  for (int k0 = 0; k0 < np; k0 += 128) {                 // (turns past the width repeat its first columns and are not used)
    f32x4 c[8], x[8];
#pragma unroll
    for (int k = 0; k < 8; k++) { const int o = k0 + 16 * k < np ? k0 + 16 * k : 0; c[k] = *reinterpret_cast<const f32x4*>(cp + o); x[k] = *reinterpret_cast<const f32x4*>(bp + o); }
#pragma unroll
    for (int k = 0; k < 8; k++) {
      if (k0 + 16 * k >= np) continue;
#pragma unroll
      for (int i = 0; i < 4; i++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(c[k][i], x[k][i], acc, 0, 0, 0);
    }
  }
  float* o = b.cb + ((int64_t)blockIdx.x * d.groups + g) * SSD_CHUNK * SSD_CHUNK;
#pragma unroll
  for (int i = 0; i < 4; i++) o[(tr * 16 + fg * 4 + i) * SSD_CHUNK + tc * 16 + fr] = acc[i];
}

// ------------------------------------------------------------------------------------------
// prompt pass 3: the walk, one work-group per (16 CT columns of a head, entry).  With S the state before the chunk,
//     y_t = exp(L_t) S^T C_t + sum_{s<=t} (C_t . B_s) exp(L_t - L_s) dt_s x_s + D x_t,
//     S <- exp(L_last) S + sum_s B_s exp(L_last - L_s) dt_s x_s^T.
// Wave w makes the outputs of the chunk's tokens 16 w .. 16 w + 15 and holds the state rows of tiles w + 4 j as matrix-core result
// registers, which pass to the other waves as operands through LDS (two copies, one barrier a chunk).  Every other operand comes
// straight from the buffers; states of up to 128 rows request it a chunk ahead (wider ones have no registers left for that).
// ------------------------------------------------------------------------------------------
template <int TPW, int CT>
__global__ __launch_bounds__(256, 1) void ssd_walk_kernel(const SsdDims d, const SsdW w, float* state, const int64_t s_elems, const StepRows r, const SsdBuf b, const int32_t* chunk0)
{
  __shared__ f32x4 sS[2][TPW * 4][CT][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), fr = lane & 15, fg = lane >> 4;
  const int slices = (d.vdim + 16 * CT - 1) / (16 * CT);
  // consecutive work-groups go to different XCDs; with heads in whole eights a head's slices stay on one
  const int h = d.heads % 8 == 0 ? (blockIdx.x & 7) + 8 * ((blockIdx.x >> 3) / slices) : blockIdx.x / slices;
  const int col = (d.heads % 8 == 0 ? (blockIdx.x >> 3) % slices : blockIdx.x % slices) * 16 * CT + fr;      // and 16 q further
  const int32_t* en = r.ent + 4 * blockIdx.y;
  const int slot = en[0], row0 = en[1], n = en[2], pos0 = en[3], ch0 = chunk0[blockIdx.y];
  const int g = h / (d.heads / d.groups), np = d.np(), xp = d.xp(), dvp = d.vdim_p(), nc = (n + SSD_CHUNK - 1) / SSD_CHUNK;
  const int ldb = d.groups * np, ldx = d.heads * xp;
  const float skip = w.D[h];
  float* Sg = state + slot * s_elems + (int64_t)h * d.state * dvp;
  f32x4 S[TPW][CT];
#pragma unroll
  for (int j = 0; j < TPW; j++)
#pragma unroll
    for (int q = 0; q < CT; q++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int rr = (wave + 4 * j) * 16 + fg * 4 + i;
        S[j][q][i] = pos0 > 0 && rr < d.state && col + 16 * q < d.vdim ? Sg[(int64_t)rr * dvp + col + 16 * q] : 0.0f;
      }
  struct In { f32x4 cf[TPW * 4], bf[TPW][4], cb[3], cbd, u[4], dt, l, a, tau; float x[CT][4][4], lt; };
  const unsigned lx = fg * 4 * ldx + col, lc = fr * SSD_CHUNK + fg * 4, lb = fr * ldb + fg * 4;
  const float* btp = b.bt + ((int64_t)ch0 * d.groups + g) * np * SSD_CHUNK;
  const float* cbp = b.cb + ((int64_t)ch0 * d.groups + g) * SSD_CHUNK * SSD_CHUNK + wave * 16 * SSD_CHUNK;
  const float* fp = b.fac + ((int64_t)ch0 * d.heads + h) * SSD_FACTORS;
  // (rows of x and C past the portion's end are other rows, or the slack behind the last one: x is replaced at use, such outputs are
  // not kept; columns past the head's width are another head's and are not kept either)
  auto fetch = [&](int c, In& v) {
    c = min(c, nc - 1);
    const int64_t rr = row0 + c * SSD_CHUNK;
    const float* cp = b.C + (rr + wave * 16) * ldb + g * np;
#pragma unroll
    for (int k = 0; k < TPW * 4; k++) v.cf[k] = *reinterpret_cast<const f32x4*>(cp + k * 16 + lb);
    const float* xb = b.x + rr * ldx + h * xp;
#pragma unroll
    for (int t = 0; t < 4; t++)
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int q = 0; q < CT; q++) v.x[q][t][i] = (xb + (t * 16 + i) * ldx + q * 16)[lx];
    const float* cbc = cbp + (int64_t)c * d.groups * SSD_CHUNK * SSD_CHUNK, *f0 = fp + (int64_t)c * d.heads * SSD_FACTORS;
#pragma unroll
    for (int t = 0; t < 3; t++) v.cb[t] = *reinterpret_cast<const f32x4*>(cbc + t * 16 + lc);
    v.cbd = *reinterpret_cast<const f32x4*>(cbc + wave * 16 + lc);
#pragma unroll
    for (int t = 0; t < 4; t++) v.u[t] = *reinterpret_cast<const f32x4*>(f0 + t * 16 + fg * 4);
    v.dt = *reinterpret_cast<const f32x4*>(f0 + 64 + wave * 16 + fg * 4); v.l = *reinterpret_cast<const f32x4*>(f0 + 128 + wave * 16 + fg * 4);
    v.a = *reinterpret_cast<const f32x4*>(f0 + 192 + wave * 16 + fg * 4); v.tau = *reinterpret_cast<const f32x4*>(f0 + 256);
    v.lt = f0[128 + wave * 16 + fr];
    const float* bp = btp + (int64_t)c * ldb * SSD_CHUNK;
#pragma unroll
    for (int j = 0; j < TPW; j++)
#pragma unroll
      for (int t = 0; t < 4; t++) v.bf[j][t] = *reinterpret_cast<const f32x4*>(bp + (wave + 4 * j) * 16 * SSD_CHUNK + t * 16 + lc);
  };
  auto chunk = [&](int c, const In& v) {
    const int nt = n - c * SSD_CHUNK;
    if (nt <= 0) return;
#pragma unroll
    for (int j = 0; j < TPW; j++)
#pragma unroll
      for (int q = 0; q < CT; q++) sS[c & 1][wave + 4 * j][q][lane] = S[j][q];
    float xl[CT][4][4];
#pragma unroll
    for (int t = 0; t < 4; t++)
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int q = 0; q < CT; q++) xl[q][t][i] = t * 16 + fg * 4 + i < nt ? v.x[q][t][i] * v.u[t][i] : 0.0f;
    __syncthreads();
    if (wave * 16 < nt) {
      f32x4 y[CT][2];
#pragma unroll
      for (int q = 0; q < CT; q++) y[q][0] = y[q][1] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int k = 0; k < TPW * 4; k++) {
        f32x4 sf[CT];
#pragma unroll
        for (int q = 0; q < CT; q++) sf[q] = sS[c & 1][k][q][lane];
#pragma unroll
        for (int i = 0; i < 4; i++)
#pragma unroll
          for (int q = 0; q < CT; q++) y[q][i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(v.cf[k][i], sf[q][i], y[q][i & 1], 0, 0, 0);
      }
      float lead = 1.0f;                                 // decay from the chunk's start to the wave's tile
#pragma unroll
      for (int t = 0; t < 3; t++) lead *= t < wave ? v.tau[t] : 1.0f;
#pragma unroll
      for (int q = 0; q < CT; q++) { y[q][0] = (y[q][0] + y[q][1]) * lead; y[q][1] = f32x4{0.0f, 0.0f, 0.0f, 0.0f}; }
      float f = 1.0f;
#pragma unroll
      for (int t = 2; t >= 0; t--) {                     // tiles before the wave's, the nearest first
        if (t >= wave) continue;
#pragma unroll
        for (int i = 0; i < 4; i++)
#pragma unroll
          for (int q = 0; q < CT; q++) y[q][i & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(v.cb[t][i] * f, xl[q][t][i], y[q][i & 1], 0, 0, 0);
        f *= v.tau[t];
      }
      float own[CT][4];
#pragma unroll
      for (int q = 0; q < CT; q++)
#pragma unroll
        for (int i = 0; i < 4; i++) own[q][i] = wave == 0 ? v.x[q][0][i] : wave == 1 ? v.x[q][1][i] : wave == 2 ? v.x[q][2][i] : v.x[q][3][i];
#pragma unroll
      for (int q = 0; q < CT; q++) y[q][0] = (y[q][0] + y[q][1]) * v.a;
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int s = fg * 4 + i;
        const bool in = wave * 16 + s < nt;
        const float gv = s <= fr ? v.cbd[i] * expf(v.lt - v.l[i]) : 0.0f;
#pragma unroll
        for (int q = 0; q < CT; q++) y[q][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(gv, in ? own[q][i] * v.dt[i] : 0.0f, y[q][0], 0, 0, 0);
      }
      float* yo = b.y + (int64_t)(row0 + c * SSD_CHUNK) * d.inner() + h * d.vdim + col;
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int q = 0; q < CT; q++) {
          const int t = wave * 16 + fg * 4 + i;
          if (t < nt && col + 16 * q < d.vdim) yo[(int64_t)t * d.inner() + 16 * q] = fmaf(skip, own[q][i], y[q][0][i]);
        }
    }
    const float all = v.tau[0] * v.tau[1] * v.tau[2] * v.tau[3];
#pragma unroll
    for (int j = 0; j < TPW; j++)
#pragma unroll
      for (int q = 0; q < CT; q++) S[j][q] *= all;
    float f = 1.0f;
#pragma unroll
    for (int t = 3; t >= 0; t--) {
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int q = 0; q < CT; q++) {
          const float xs = xl[q][t][i] * f;
#pragma unroll
          for (int j = 0; j < TPW; j++) S[j][q] = __builtin_amdgcn_mfma_f32_16x16x4f32(v.bf[j][t][i], xs, S[j][q], 0, 0, 0);
        }
      f *= v.tau[t];
    }
  };
  if constexpr (TPW <= 2) {
    In va, vb;
    fetch(0, va);
    for (int c = 0; c < nc; c += 2) {
      fetch(c + 1, vb);
      __builtin_amdgcn_sched_barrier(0);
      chunk(c, va);
      fetch(c + 2, va);
      __builtin_amdgcn_sched_barrier(0);
      chunk(c + 1, vb);
    }
  } else {
    In v;
    for (int c = 0; c < nc; c++) { fetch(c, v); chunk(c, v); }
  }
#pragma unroll
  for (int j = 0; j < TPW; j++)
#pragma unroll
    for (int q = 0; q < CT; q++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int rr = (wave + 4 * j) * 16 + fg * 4 + i;
        if (rr < d.state && col + 16 * q < dvp) Sg[(int64_t)rr * dvp + col + 16 * q] = S[j][q][i];
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
// gate, then RMS norm of each of norm_groups equal parts, gain.  Up to VALUES values a thread stay in registers (four at a time when the
// parts' widths allow); wider parts are made again.  The first part's work-group of a portion's last rows also keeps their raw inputs (a
// decoded token's are kept already).
// ------------------------------------------------------------------------------------------
template <typename AT, bool VEC>
__global__ __launch_bounds__(1024) void ssd_finish_kernel(const SsdDims d, const SsdIn in, const SsdW w, float* hist, const int64_t h_elems, const StepRows r, const float* y, const int single, AT* out, const int64_t ldo)
{
  constexpr int VALUES = 8, PER = VEC ? 4 : 1, TURNS = VALUES / PER;
  __shared__ float part[16];
  const int64_t row = blockIdx.x;
  const int tid = threadIdx.x, inner = d.inner(), gw = inner / d.norm_groups, c0 = blockIdx.y * gw;
  const float *p = in.proj + row * in.ldp, *yr = y + row * inner + c0, *z = p + in.oz + c0, *gain = w.norm + c0;
  AT* o = out + row * ldo + c0;
  float u[TURNS][PER], s = 0.0f;
  auto load = [&](const float* a, int c, float* v) {
    if constexpr (VEC) *reinterpret_cast<f32x4*>(v) = *reinterpret_cast<const f32x4*>(a + c);
    else v[0] = a[c];
  };
  auto gated = [&](int c, float* v) {
    float t[PER];
    load(yr, c, v); load(z, c, t);
#pragma unroll
    for (int i = 0; i < PER; i++) v[i] *= t[i] * sigmoid_f(t[i]);
  };
#pragma unroll
  for (int i = 0; i < TURNS; i++) {
    const int c = (tid + i * 1024) * PER;
    if (c < gw) {
      gated(c, u[i]);
#pragma unroll
      for (int k = 0; k < PER; k++) s = fmaf(u[i][k], u[i][k], s);
    }
  }
  for (int c = (tid + TURNS * 1024) * PER; c < gw; c += 1024 * PER) {
    float v[PER];
    gated(c, v);
#pragma unroll
    for (int k = 0; k < PER; k++) s = fmaf(v[k], v[k], s);
  }
  s = wave_total(s);
  if ((tid & 63) == 0) part[tid >> 6] = s;
  __syncthreads();
  s = 0.0f;
#pragma unroll
  for (int i = 0; i < 16; i++) s += part[i];
  const float inv = 1.0f / sqrtf(s / (float)gw + d.eps);
  auto put = [&](int c, const float* v) {
    float t[PER];
    load(gain, c, t);
#pragma unroll
    for (int k = 0; k < PER; k++) t[k] *= v[k] * inv;
    if constexpr (VEC && sizeof(AT) == 2) *reinterpret_cast<uint2*>(o + c) = make_uint2(bf16_bits(t[0]) | (uint32_t)bf16_bits(t[1]) << 16, bf16_bits(t[2]) | (uint32_t)bf16_bits(t[3]) << 16);
    else {
#pragma unroll
      for (int k = 0; k < PER; k++) o[c + k] = (AT)t[k];
    }
  };
#pragma unroll
  for (int i = 0; i < TURNS; i++) { const int c = (tid + i * 1024) * PER; if (c < gw) put(c, u[i]); }
  for (int c = (tid + TURNS * 1024) * PER; c < gw; c += 1024 * PER) { float v[PER]; gated(c, v); put(c, v); }
  if (!single && blockIdx.y == 0 && r.last[row] - row < d.taps) {
    const int C = d.channels();
    float* ring = hist + r.slot[row] * h_elems + (int64_t)(r.pos[row] % d.taps) * C;
    for (int c = tid; c < C; c += 1024) ring[c] = p[in.ox + c];
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
  hipLaunchKernelGGL(ssd_chunk_kernel, dim3(n_chunks, 2 * d.groups + (d.heads + SCORE_WAVES - 1) / SCORE_WAVES), dim3(64 * SCORE_WAVES), 0, ctx().stream, d, r, w, b, chunks);
#define WALK(N, CT) hipLaunchKernelGGL((ssd_walk_kernel<N, CT>), dim3((d.vdim + 16 * CT - 1) / (16 * CT) * d.heads, r.n_ent), dim3(256), 0, ctx().stream, d, w, st.S, st.s_elems, r, b, chunk0)
#define WALK_N(N) do { if (d.vdim > 16) WALK(N, 2); else WALK(N, 1); } while (0)
  const int tpw = d.np() / 64;
  if (tpw == 1) WALK_N(1); else if (tpw == 2) WALK_N(2); else if (tpw == 3) WALK(3, 1); else WALK(4, 1);
#undef WALK_N
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
  const bool vec = d.inner() / d.norm_groups % 4 == 0 && in.oz % 4 == 0 && in.ldp % 4 == 0 && ldo % 4 == 0;
#define FINISH(AT, V) hipLaunchKernelGGL((ssd_finish_kernel<AT, V>), grid, dim3(1024), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b.y, single ? 1 : 0, (AT*)out, ldo)
  if (act_t == ACT_T_BF16) { if (vec) FINISH(bf16_t, true); else FINISH(bf16_t, false); }
  else { if (vec) FINISH(float, true); else FINISH(float, false); }
#undef FINISH
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

}  // namespace cai
