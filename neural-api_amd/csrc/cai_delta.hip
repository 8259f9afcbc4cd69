// Gated delta rule with short convolutions: prompt kernels (convolution and unit norms, the scan, the gated output norm) and a
// one-launch decode kernel.
//
// Per head a float state S [dim][vdim] (rows padded to four columns, the padding stays zero); one token does  S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.
// With S' = diag(g) S the read-out is  o = S'^T q + (q . k) u, so both products with S' are taken together and the second
// reduction is off the dependent chain.  Everything that touches the state is 32-bit.
#include "cai_layered.hpp"
#include "cai_recurrent.hpp"

namespace cai {

// ------------------------------------------------------------------------------------------
// prompt pass 1: q and k unit vectors (q scaled), v, decay, write strength, q . k.
// A wave owns one unit - the q and k channels of a key head, 256 channels of v, 256 decays, the write strengths - over eight
// consecutive rows; the convolution slides over them, so each input is fetched once (TAPS = 4; other lengths look back per row).
// ------------------------------------------------------------------------------------------
constexpr int PREP_ROWS = 8;

template <int TAPS>
__global__ __launch_bounds__(256) void delta_prep_kernel(const DeltaDims d, const DeltaIn in, const DeltaW w, const float* hist, const int64_t h_elems, const StepRows r, const DeltaBuf b)
{
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r0 = blockIdx.x * PREP_ROWS, r1 = min(r0 + PREP_ROWS, r.n_rows);
  const int C = d.channels(), kw = d.kv_heads * d.dim, vw = d.heads * d.vdim, bw = d.heads + d.kv_heads;
  const int gw = d.channel_decay ? d.heads * d.dim : d.heads;
  const int nv = (vw + 255) / 256, ng = (gw + 255) / 256;
  int unit = blockIdx.y * 4 + wave;
  if (unit < d.kv_heads) {
    const int g = unit, c0 = g * d.dim;
    const float qs = rsqrtf((float)d.dim);
    ConvWindow<TAPS ? TAPS : 2> wq, wk;
    if (TAPS) { wq.taps(w.cq, c0, lane, d.dim); wk.taps(w.ck, c0, lane, d.dim); }
    for (int row = r0; row < r1; row++) {
      const int pos = r.pos[row], back = row - r.first[row];
      const float* ring = hist + r.slot[row] * h_elems;
      const float* p = in.proj + row * in.ldp;
      if (TAPS && (row == r0 || back == 0)) {
        wq.history(p + in.oq, in.ldp, back, pos, ring, C, 0, c0, lane, d.dim);
        wk.history(p + in.ok, in.ldp, back, pos, ring, C, kw, c0, lane, d.dim);
      }
      float q[4], k[4], sq = 0.0f, sk = 0.0f, dot = 0.0f;
#pragma unroll
      for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; q[i] = c < d.dim ? p[in.oq + c0 + c] : 0.0f; k[i] = c < d.dim ? p[in.ok + c0 + c] : 0.0f; }
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int c = lane + 64 * i;
        if (i * 64 >= d.dim) continue;
        if (TAPS) { q[i] = wq.step(i, q[i]); k[i] = wk.step(i, k[i]); }
        else if (c < d.dim) {
          q[i] = conv_silu(p + in.oq, in.ldp, back, pos, ring, C, 0, w.cq, d.taps, c0 + c);
          k[i] = conv_silu(p + in.ok, in.ldp, back, pos, ring, C, kw, w.ck, d.taps, c0 + c);
        }
        sq = fmaf(q[i], q[i], sq); sk = fmaf(k[i], k[i], sk); dot = fmaf(q[i], k[i], dot);
      }
      const float nq = qs / sqrtf(wave_total(sq) + 1e-6f), nk = 1.0f / sqrtf(wave_total(sk) + 1e-6f);
      dot = wave_total(dot) * nq * nk;
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int c = lane + 64 * i;
        if (c < d.dim) { b.q[(int64_t)row * kw + c0 + c] = q[i] * nq; b.k[(int64_t)row * kw + c0 + c] = k[i] * nk; }
      }
      if (lane == 0) b.beta[(int64_t)row * bw + d.heads + g] = dot;
    }
    return;
  }
  unit -= d.kv_heads;
  if (unit < nv) {
    const int c0 = unit * 256, n = min(256, vw - c0);
    ConvWindow<TAPS ? TAPS : 2> wv;
    if (TAPS) wv.taps(w.cv, c0, lane, n);
    for (int row = r0; row < r1; row++) {
      const int pos = r.pos[row], back = row - r.first[row];
      const float* ring = hist + r.slot[row] * h_elems;
      const float* p = in.proj + row * in.ldp + in.ov;
      if (TAPS && (row == r0 || back == 0)) wv.history(p, in.ldp, back, pos, ring, C, 2 * kw, c0, lane, n);
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int c = lane + 64 * i;
        if (TAPS) { const float v = wv.step(i, c < n ? p[c0 + c] : 0.0f); if (c < n) b.v[(int64_t)row * vw + c0 + c] = v; }
        else if (c < n) b.v[(int64_t)row * vw + c0 + c] = conv_silu(p, in.ldp, back, pos, ring, C, 2 * kw, w.cv, d.taps, c0 + c);
      }
    }
    return;
  }
  unit -= nv;
  if (unit < ng) {
    for (int i = 0; i < 4; i++) {
      const int c = unit * 256 + lane + 64 * i;
      if (c >= gw) continue;
      const float bias = w.dt_bias[c], rate = w.rate[d.channel_decay ? c / d.dim : c];
#pragma unroll
      for (int u = 0; u < PREP_ROWS; u++) {
        const int row = min(r0 + u, r1 - 1);
        const float z = d.rank_a ? b.za[(int64_t)row * gw + c] : in.proj[row * in.ldp + in.oa + c];
        b.g[(int64_t)row * gw + c] = expf(rate * softplus_f(z + bias));
      }
    }
    return;
  }
  if (unit == ng)
    for (int row = r0; row < r1; row++)
      for (int h = lane; h < d.heads; h += 64) b.beta[(int64_t)row * bw + h] = sigmoid_f(in.proj[row * in.ldp + in.ob + h]);
}

// ------------------------------------------------------------------------------------------
// prompt pass 2 for short portions: the scan.  A wave owns four columns of one head's state: 16 lanes a column, RPL rows a lane (rows
// 64 j + 4 (lane & 15) + i), in registers for the whole portion.  Tokens are staged through LDS 16 at a time, the next block
// requested before the current one is walked; the walk itself has no barrier.
// ------------------------------------------------------------------------------------------
constexpr int SCAN_TB = 16;
template <int RPL, bool CH>
__global__ __launch_bounds__(256) void delta_scan_kernel(const DeltaDims d, float* state, const int64_t s_elems, const StepRows r, const DeltaBuf b)
{
  constexpr int DP = RPL * 16;
  __shared__ f32x4 sq[SCAN_TB][DP / 4], sk[SCAN_TB][DP / 4], sg[CH ? SCAN_TB : 1][CH ? DP / 4 : 1];
  __shared__ float sv[SCAN_TB][16], so[SCAN_TB][16], sgs[SCAN_TB], sb[SCAN_TB], sqk[SCAN_TB];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c0 = blockIdx.x * 16, h = blockIdx.y;
  const int32_t* en = r.ent + 4 * blockIdx.z;
  const int slot = en[0], row0 = en[1], n = en[2], pos0 = en[3];
  const int g = h / (d.heads / d.kv_heads), kw = d.kv_heads * d.dim, vw = d.heads * d.vdim, gw = d.heads * d.dim, bw = d.heads + d.kv_heads;
  const int rg = lane & 15, cl = wave * 4 + (lane >> 4), col = c0 + cl;
  const int dvp = d.vdim_p();
  float* Sg = state + slot * s_elems + (int64_t)h * d.dim * dvp;
  float S[RPL];
#pragma unroll
  for (int j = 0; j < RPL; j++) {
    const int rr = (j >> 2) * 64 + rg * 4 + (j & 3);
    S[j] = pos0 > 0 && rr < d.dim && col < d.vdim ? Sg[(int64_t)rr * dvp + col] : 0.0f;
  }
  float nq[RPL], nk[RPL], ng[CH ? RPL : 1], nv, nb, nqk, ngs;
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < RPL; i++) {
      const int e = tid + 256 * i, t = t0 + e / DP, c = e % DP;
      const bool ok = t < n && c < d.dim;
      const int64_t rw = row0 + (ok ? t : 0);
      const int cc = ok ? c : 0;
      nq[i] = b.q[rw * kw + g * d.dim + cc]; nk[i] = b.k[rw * kw + g * d.dim + cc];
      if (CH) ng[i] = b.g[rw * gw + h * d.dim + cc];
      if (!ok) { nq[i] = 0.0f; nk[i] = 0.0f; }
    }
    {
      const int t = t0 + (tid >> 4), c = c0 + (tid & 15);
      nv = t < n && c < d.vdim ? b.v[(int64_t)(row0 + t) * vw + h * d.vdim + c] : 0.0f;
    }
    if (tid < SCAN_TB) {
      const int64_t rw = row0 + min(t0 + tid, n - 1);
      nb = b.beta[rw * bw + h]; nqk = b.beta[rw * bw + d.heads + g];
      if (!CH) ngs = b.g[rw * d.heads + h];
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += SCAN_TB) {
#pragma unroll
    for (int i = 0; i < RPL; i++) {
      const int e = tid + 256 * i, t = e / DP, c = e % DP;
      reinterpret_cast<float*>(sq[t])[c] = nq[i]; reinterpret_cast<float*>(sk[t])[c] = nk[i];
      if (CH) reinterpret_cast<float*>(sg[t])[c] = ng[i];
    }
    sv[tid >> 4][tid & 15] = nv;
    if (tid < SCAN_TB) { sb[tid] = nb; sqk[tid] = nqk; if (!CH) sgs[tid] = ngs; }
    __syncthreads();
    if (t0 + SCAN_TB < n) fetch(t0 + SCAN_TB);
    const int nt = min(SCAN_TB, n - t0);
    auto token = [&](int t) {
      float ks = 0.0f, qd = 0.0f;
      f32x4 kf[RPL / 4];
#pragma unroll
      for (int j = 0; j < RPL / 4; j++) {
        kf[j] = sk[t][j * 16 + rg];
        const f32x4 qf = sq[t][j * 16 + rg];
        f32x4 gf;
        if (CH) gf = sg[t][j * 16 + rg];
        else { const float s = sgs[t]; gf = f32x4{s, s, s, s}; }
#pragma unroll
        for (int i = 0; i < 4; i++) {
          S[j * 4 + i] *= gf[i];
          ks = fmaf(S[j * 4 + i], kf[j][i], ks); qd = fmaf(S[j * 4 + i], qf[i], qd);
        }
      }
      ks = row16_total(ks); qd = row16_total(qd);
      const float u = sb[t] * (sv[t][cl] - ks);
#pragma unroll
      for (int j = 0; j < RPL / 4; j++)
#pragma unroll
        for (int i = 0; i < 4; i++) S[j * 4 + i] = fmaf(kf[j][i], u, S[j * 4 + i]);
      if (rg == 0) so[t][cl] = fmaf(sqk[t], u, qd);
    };
    if (nt == SCAN_TB) {
#pragma unroll 4
      for (int t = 0; t < SCAN_TB; t++) token(t);
    } else for (int t = 0; t < nt; t++) token(t);
    __syncthreads();
    {
      const int t = tid >> 4, c = c0 + (tid & 15);
      if (t < nt && c < d.vdim) b.o[(int64_t)(row0 + t0 + t) * vw + h * d.vdim + c] = so[t][tid & 15];
    }
  }
#pragma unroll
  for (int j = 0; j < RPL; j++) {
    const int rr = (j >> 2) * 64 + rg * 4 + (j & 3);
    if (rr < d.dim && col < dvp) Sg[(int64_t)rr * dvp + col] = S[j];
  }
}

// ------------------------------------------------------------------------------------------
// prompt pass 2 for long portions: the same recurrence in chunks of 16 tokens, on the float matrix cores (32-bit throughout).
//
// With P_t the product of the decays of the chunk's tokens up to t, D_ts that of the tokens after s up to t, and S the state
// before the chunk, the writes u of a chunk solve a unit lower triangular system,
//     u_t = beta_t (v_t - S^T (P_t k_t) - sum_{s<t} A_ts u_s),   A_ts = k_t . D_ts k_s,
// so with T = (I + diag(beta) A)^-1 diag(beta):   U = T V - (T [P k]) S =: U0 - W S.   Then
//     o_t = S^T (P_t q_t) + sum_{s<=t} (q_t . D_ts k_s) u_s,      S <- P_16 S + sum_s (D_16,s k_s) u_s^T.
// Everything before "S" is made for all chunks at once (first kernel); the second kernel walks the chunks of a sequence with a
// 16-column slice of the state in registers.  Decays enter only as running products, never as quotients or differences of
// logarithms, so strong decay costs no accuracy.
// ------------------------------------------------------------------------------------------
constexpr int CHUNK = DELTA_CHUNK;

template <bool CH>
__global__ __launch_bounds__(256) void delta_chunk_kernel(const DeltaDims d, const StepRows r, const DeltaBuf b, const int32_t* chunks)
{
  extern __shared__ float lds[];
  __shared__ float sA[CHUNK][CHUNK + 1], sQ[CHUNK][CHUNK + 1], sP[CH ? 1 : 4][CHUNK][CHUNK + 1];
  __shared__ f32x4 sT[CHUNK][CHUNK / 4];
  __shared__ float sbeta[CHUNK], sg1[CHUNK], sdot[CHUNK];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), fr = lane & 15, fg = lane >> 4;
  const int32_t* en = r.ent + 4 * chunks[2 * blockIdx.x];
  const int t0 = chunks[2 * blockIdx.x + 1], nt = min(CHUNK, en[2] - t0), h = blockIdx.y;
  const int64_t row0 = en[1] + t0;
  const int g = h / (d.heads / d.kv_heads), kw = d.kv_heads * d.dim, vw = d.heads * d.vdim, gw = d.heads * d.dim, bw = d.heads + d.kv_heads;
  const int dp = (d.dim + 15) & ~15, DS = dp + 4;
  float *sk = lds, *sq = lds + CHUNK * DS, *sg = lds + 2 * CHUNK * DS;       // sg: channel decays, later their running products
  for (int e = tid; e < CHUNK * dp; e += 256) {
    const int t = e / dp, c = e - t * dp;
    const bool ok = t < nt && c < d.dim;
    const int64_t rw = row0 + (ok ? t : 0); const int cc = ok ? c : 0;
    const float k = b.k[rw * kw + g * d.dim + cc], q = b.q[rw * kw + g * d.dim + cc];
    sk[t * DS + c] = ok ? k : 0.0f; sq[t * DS + c] = ok ? q : 0.0f;
    if (CH) { const float x = b.g[rw * gw + h * d.dim + cc]; sg[t * DS + c] = ok ? x : 1.0f; }
  }
  if (tid < CHUNK) {
    const bool ok = tid < nt; const int64_t rw = row0 + (ok ? tid : 0);
    sbeta[tid] = ok ? b.beta[rw * bw + h] : 0.0f; sdot[tid] = ok ? b.beta[rw * bw + d.heads + g] : 0.0f;
    sg1[tid] = !CH && ok ? b.g[rw * d.heads + h] : 1.0f;
  }
  __syncthreads();
  if (CH) {
    // thread (s, 16 channel lanes): running product of the decays after s
    const int s = tid >> 4, cl = tid & 15;
    float a[CHUNK], o[CHUNK];
#pragma unroll
    for (int t = 0; t < CHUNK; t++) a[t] = o[t] = 0.0f;
    for (int c = cl; c < dp; c += 16) {
      const float ks = sk[s * DS + c];
      float e = ks;
#pragma unroll
      for (int t = 1; t < CHUNK; t++) {
        e = t > s ? e * sg[t * DS + c] : e;
        a[t] = fmaf(sk[t * DS + c], e, a[t]); o[t] = fmaf(sq[t * DS + c], e, o[t]);
      }
    }
#pragma unroll
    for (int t = 0; t < CHUNK; t++) {
      const float x = row16_total(a[t]), y = row16_total(o[t]);
      if (cl == 0) { sA[t][s] = t > s ? x : 0.0f; sQ[t][s] = t > s ? y : t == s ? sdot[t] : 0.0f; }
    }
    __syncthreads();
    // k times the decays behind it (in place of the decays), q times those up to it, the chunk's whole decay
    for (int c = tid; c < dp; c += 256) {
      float z = 1.0f;
      float gr[CHUNK];
#pragma unroll
      for (int t = CHUNK - 1; t >= 0; t--) {
        gr[t] = sg[t * DS + c];
        if (t < nt && c < d.dim) b.g[(row0 + t) * gw + h * d.dim + c] = sk[t * DS + c] * z;
        z *= gr[t];
      }
      float p = 1.0f;
#pragma unroll
      for (int t = 0; t < CHUNK; t++) {
        p *= gr[t];
        sg[t * DS + c] = p;
        if (t < nt && c < d.dim) b.qt[(row0 + t) * gw + h * d.dim + c] = sq[t * DS + c] * p;
      }
      if (c < d.dim) b.gt[(int64_t)blockIdx.x * gw + h * d.dim + c] = p;
    }
  } else {
    // K K^T and Q K^T, half of the width by each of two waves
    f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
    const float* am = wave & 1 ? sq : sk;
    for (int kt = wave >> 1; kt < dp / 16; kt += 2) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(am + fr * DS + kt * 16 + fg * 4), y = *reinterpret_cast<const f32x4*>(sk + fr * DS + kt * 16 + fg * 4);
#pragma unroll
      for (int i = 0; i < 4; i++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[i], y[i], acc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) sP[wave][fg * 4 + i][fr] = acc[i];
    __syncthreads();
    const int t = tid >> 4, s = tid & 15;
    float e = t >= s ? 1.0f : 0.0f;
#pragma unroll
    for (int x = 1; x < CHUNK; x++) e *= x > s && x <= t ? sg1[x] : 1.0f;
    sA[t][s] = t > s ? e * (sP[0][t][s] + sP[2][t][s]) : 0.0f;
    sQ[t][s] = e * (sP[1][t][s] + sP[3][t][s]);
    if (tid < nt) {
      float p = 1.0f, z = 1.0f;
#pragma unroll
      for (int x = 0; x < CHUNK; x++) { p *= x <= tid ? sg1[x] : 1.0f; z *= x > tid ? sg1[x] : 1.0f; }
      float* o = b.gt + ((row0 + tid) * d.heads + h) * 2;
      o[0] = p; o[1] = z;
    }
  }
  __syncthreads();
  {
    const int t = tid >> 4, s = tid & 15;
    if (t < nt) b.qk[((row0 + t) * d.heads + h) * CHUNK + s] = sQ[t][s];
  }
  if (tid < CHUNK) {                       // column tid of T by forward substitution
    float c[CHUNK];
#pragma unroll
    for (int t = 0; t < CHUNK; t++) {
      float x = t == tid ? 1.0f : 0.0f;
#pragma unroll
      for (int s = 0; s < t; s++) x = fmaf(-sA[t][s], c[s], x);
      c[t] = x * sbeta[t];
      reinterpret_cast<float*>(sT[t])[tid] = c[t];
    }
  }
  if (!CH && tid >= 64 && tid < 64 + CHUNK) {            // running products for T [P k]
    float p = 1.0f;
    for (int x = 0; x <= tid - 64; x++) p *= sg1[x];
    sdot[tid - 64] = p;
  }
  __syncthreads();
  const f32x4 tf = sT[fr][fg];
  for (int ct = wave; ct < dp / 16; ct += 4) {           // W = T [P k]
    f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
    const int c = ct * 16 + fr;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int s = fg * 4 + i;
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(tf[i], sk[s * DS + c] * (CH ? sg[s * DS + c] : sdot[s]), acc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) if (fg * 4 + i < nt && c < d.dim) b.w[(row0 + fg * 4 + i) * gw + h * d.dim + c] = acc[i];
  }
  for (int ct = wave; ct * 16 < d.vdim; ct += 4) {       // U0 = T V, in place of V
    f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
    const int c = ct * 16 + fr;
    float x[4];
#pragma unroll
    for (int i = 0; i < 4; i++) x[i] = fg * 4 + i < nt && c < d.vdim ? b.v[(row0 + fg * 4 + i) * vw + h * d.vdim + c] : 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(tf[i], x[i], acc, 0, 0, 0);
#pragma unroll
    for (int i = 0; i < 4; i++) if (fg * 4 + i < nt && c < d.vdim) b.v[(row0 + fg * 4 + i) * vw + h * d.vdim + c] = acc[i];
  }
}

// The walk: one work-group per (16 value columns, head, entry).  Waves 0 .. NW - 1 hold the state - wave w the key rows of tiles
// w TPW .. as matrix-core result registers, which are at the same time the right operand of the products with S - and wave NW makes
// the output: it contributes U0 to the sum of a chunk's writes and finishes the previous chunk's rows of o while the others are a
// chunk further.  One barrier a chunk; the partial sums live in LDS for three chunks.
template <int NW, int TPW, bool CH, bool VEC>      // VEC: the key width is a multiple of four
__global__ __launch_bounds__(64 * (NW + 1)) void delta_walk_kernel(const DeltaDims d, float* state, const int64_t s_elems, const StepRows r, const DeltaBuf b, const int32_t* chunk0)
{
  __shared__ f32x4 pu[3][NW + 1][64], po[3][NW][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), fr = lane & 15, fg = lane >> 4;
  // consecutive work-groups go to different XCDs; the column slices of a head read the same chunk data, so with heads in whole
  // eights every head stays on one XCD (and in its L2)
  const int slices = (d.vdim + 15) / 16;
  const int h = d.heads % 8 == 0 ? (blockIdx.x & 7) + 8 * ((blockIdx.x >> 3) / slices) : blockIdx.x / slices;
  const int col = (d.heads % 8 == 0 ? (blockIdx.x >> 3) % slices : blockIdx.x % slices) * 16 + fr;
  const int32_t* en = r.ent + 4 * blockIdx.y;
  const int slot = en[0], row0 = en[1], n = en[2], pos0 = en[3], ch0 = chunk0[blockIdx.y];
  const int g = h / (d.heads / d.kv_heads), kw = d.kv_heads * d.dim, vw = d.heads * d.vdim, gw = d.heads * d.dim, dvp = d.vdim_p();
  const int nc = (n + CHUNK - 1) / CHUNK;
  auto total = [&](int it) -> f32x4 {                    // a chunk's writes: U0 and every wave's part of - W S
    f32x4 x[NW];
#pragma unroll
    for (int v = 0; v < NW; v++) x[v] = pu[it][v][lane];
    x[0] += pu[it][NW][lane];
#pragma unroll
    for (int m = NW / 2; m; m >>= 1)
#pragma unroll
      for (int v = 0; v < m; v++) x[v] += x[v + m];
    return x[0];
  };
  if (wave == NW) {
    const unsigned lv = fg * 4 * vw + min(col, d.vdim - 1), lqk = fr * d.heads * CHUNK + fg * 4, lo = fg * 4 * vw + col;
    struct Out { f32x4 u0, qk; };
    auto fetch = [&](int c, Out& x) {
      const int64_t rr = row0 + min(c, nc - 1) * CHUNK;
      const float* vb = b.v + rr * vw + h * d.vdim;
#pragma unroll
      for (int i = 0; i < 4; i++) x.u0[i] = (vb + i * vw)[lv];
      x.qk = *reinterpret_cast<const f32x4*>(b.qk + (rr * d.heads + h) * CHUNK + lqk);
    };
    f32x4 qk_last = {0.0f, 0.0f, 0.0f, 0.0f};
    auto finish = [&](int c, int it) {                   // rows of o of chunk c (parts it)
      f32x4 o = po[it][0][lane];
#pragma unroll
      for (int v = 1; v < NW; v++) o += po[it][v][lane];
      const f32x4 u = total(it);
#pragma unroll
      for (int i = 0; i < 4; i++) o = __builtin_amdgcn_mfma_f32_16x16x4f32(qk_last[i], u[i], o, 0, 0, 0);
      const int nt = n - c * CHUNK;
      if (c < 0) return;
      float* ob = b.o + (int64_t)(row0 + c * CHUNK) * vw + h * d.vdim;
#pragma unroll
      for (int i = 0; i < 4; i++) if (fg * 4 + i < nt && col < d.vdim) (ob + i * vw)[lo] = o[i];
    };
    auto chunk = [&](int c, const Out& x, int it) {
      const int nt = n - c * CHUNK;
      f32x4 u;
#pragma unroll
      for (int i = 0; i < 4; i++) u[i] = fg * 4 + i < nt && col < d.vdim ? x.u0[i] : 0.0f;
      pu[it][NW][lane] = u;
      __syncthreads();
      finish(c - 1, (it + 2) % 3);
#pragma unroll
      for (int i = 0; i < 4; i++) qk_last[i] = fr < nt ? x.qk[i] : 0.0f;
    };
    Out xa, xb, xc;
    fetch(0, xa); fetch(1, xb);
    for (int c = 0; c < nc; c += 3) {
      fetch(c + 2, xc); chunk(c, xa, 0);
      fetch(c + 3, xa); chunk(c + 1, xb, 1);
      fetch(c + 4, xb); chunk(c + 2, xc, 2);
    }
    __syncthreads();
    finish((nc + 2) / 3 * 3 - 1, 2);
    return;
  }
  float* Sg = state + slot * s_elems + (int64_t)h * d.dim * dvp;
  f32x4 S[TPW];
#pragma unroll
  for (int j = 0; j < TPW; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int c = (wave * TPW + j) * 16 + fg * 4 + i;
      S[j][i] = pos0 > 0 && c < d.dim && col < d.vdim ? Sg[(int64_t)c * dvp + col] : 0.0f;
    }
  // A chunk's inputs are requested two chunks ahead and stay as they come until they are used: arithmetic on them here would wait
  // for them here, and so would a request under a branch where the paths join.  A request is a scalar base of the chunk plus a lane
  // offset that never changes; rows past the portion's end (of another entry, or of the slack behind the last row) and columns past
  // the width are replaced by zeros at use.
  struct In { f32x4 w[TPW], q[TPW], k[TPW], tot[TPW]; float p, all, kz[4]; };
  bool ok4[TPW][VEC ? 1 : 4], ok1[TPW];
  unsigned lw[TPW], lq[TPW], lk[TPW], lt[TPW];
#pragma unroll
  for (int j = 0; j < TPW; j++) {
    const int c4 = (wave * TPW + j) * 16 + fg * 4, c1 = (wave * TPW + j) * 16 + fr;
    ok1[j] = c1 < d.dim;
#pragma unroll
    for (int i = 0; i < (VEC ? 1 : 4); i++) ok4[j][i] = c4 + i < d.dim;
    lt[j] = c4 < d.dim ? c4 : 0;
    lw[j] = fr * gw + lt[j]; lq[j] = fr * (CH ? gw : kw) + lt[j];
    lk[j] = fg * 4 * (CH ? gw : kw) + (ok1[j] ? c1 : 0);
  }
  const unsigned lp = fr * d.heads * 2, lz = fg * 4 * d.heads * 2 + 1;
  auto four = [&](const float* p, unsigned c) -> f32x4 {
    if (VEC) return *reinterpret_cast<const f32x4*>(p + c);
    return f32x4{p[c], p[c + 1], p[c + 2], p[c + 3]};                     // (may run into the next row: replaced at use)
  };
  auto fetch = [&](int c, In& x) {
    const int cc = min(c, nc - 1);
    const int64_t rr = row0 + cc * CHUNK;
    const float *wb = b.w + rr * gw + h * d.dim, *qb = CH ? b.qt + rr * gw + h * d.dim : b.q + rr * kw + g * d.dim;
    const float *kb = CH ? b.g + rr * gw + h * d.dim : b.k + rr * kw + g * d.dim, *tb = b.gt + (int64_t)(ch0 + cc) * gw + h * d.dim;
    const int ks = CH ? gw : kw;
#pragma unroll
    for (int j = 0; j < TPW; j++) {
      x.w[j] = four(wb, lw[j]); x.q[j] = four(qb, lq[j]);
#pragma unroll
      for (int i = 0; i < 4; i++) x.k[j][i] = (kb + i * ks)[lk[j]];
      if (CH) x.tot[j] = four(tb, lt[j]);
    }
    if (!CH) {
      const float* pz = b.gt + (rr * d.heads + h) * 2;
      x.p = pz[lp]; x.all = pz[(min(CHUNK, n - cc * CHUNK) - 1) * d.heads * 2];
#pragma unroll
      for (int i = 0; i < 4; i++) x.kz[i] = (pz + i * d.heads * 2)[lz];
    }
  };
  auto chunk = [&](int c, const In& x, int it) {         // (a chunk past the last one changes nothing)
    const int nt = n - c * CHUNK;
    const bool rok = fr < nt;
    f32x4 u[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}}, o = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int j = 0; j < TPW; j++)
        u[(i * TPW + j) & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(rok && ok4[j][VEC ? 0 : i] ? -x.w[j][i] : 0.0f, S[j][i], u[(i * TPW + j) & 1], 0, 0, 0);
    pu[it][wave][lane] = u[0] + u[1];
    __syncthreads();
    const f32x4 t = total(it);
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int j = 0; j < TPW; j++) {      // the read-out with the state before the chunk, while the sums arrive
        const float q = rok && ok4[j][VEC ? 0 : i] ? (CH ? x.q[j][i] : x.q[j][i] * x.p) : 0.0f;
        o = __builtin_amdgcn_mfma_f32_16x16x4f32(q, S[j][i], o, 0, 0, 0);
      }
    po[it][wave][lane] = o;
#pragma unroll
    for (int j = 0; j < TPW; j++)
#pragma unroll
      for (int i = 0; i < 4; i++) S[j][i] *= nt > 0 ? (CH ? x.tot[j][i] : x.all) : 1.0f;
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int j = 0; j < TPW; j++) {
        const float k = fg * 4 + i < nt && ok1[j] ? (CH ? x.k[j][i] : x.k[j][i] * x.kz[i]) : 0.0f;
        S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(k, t[i], S[j], 0, 0, 0);
      }
  };
  // (the scheduling barriers keep a chunk's requests in front of the chunk that is worked on: they are used two chunks later)
  In xa, xb, xc;
  fetch(0, xa); fetch(1, xb);
  for (int c = 0; c < nc; c += 3) {
    fetch(c + 2, xc);
    __builtin_amdgcn_sched_barrier(0);
    chunk(c, xa, 0);
    fetch(c + 3, xa);
    __builtin_amdgcn_sched_barrier(0);
    chunk(c + 1, xb, 1);
    fetch(c + 4, xb);
    __builtin_amdgcn_sched_barrier(0);
    chunk(c + 2, xc, 2);
  }
  __syncthreads();                         // the last chunk's read-outs are there
#pragma unroll
  for (int j = 0; j < TPW; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int c = (wave * TPW + j) * 16 + fg * 4 + i;
      if (c < d.dim && col < dvp) Sg[(int64_t)c * dvp + col] = S[j][i];
    }
}

// ------------------------------------------------------------------------------------------
// prompt pass 3: per row and head RMS norm, gain, gate; then the row's raw inputs into the ring if the portion's last taps reach it
// ------------------------------------------------------------------------------------------
template <typename AT>
__global__ __launch_bounds__(256) void delta_finish_kernel(const DeltaDims d, const DeltaIn in, const DeltaW w, float* hist, const int64_t h_elems, const StepRows r, const DeltaBuf b, AT* out, const int64_t ldo)
{
  const int row = blockIdx.x, lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int vw = d.heads * d.vdim;
  const float* p = in.proj + row * in.ldp;
  const float* gate = d.rank_g ? b.zg + (int64_t)row * vw : p + in.og;
  for (int h = wave; h < d.heads; h += 4) {
    float o[4], s = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int c = lane + 64 * i;
      o[i] = c < d.vdim ? b.o[(int64_t)row * vw + h * d.vdim + c] : 0.0f;
      s = fmaf(o[i], o[i], s);
    }
    const float inv = 1.0f / sqrtf(wave_total(s) / (float)d.vdim + d.eps);
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int c = lane + 64 * i;
      if (c < d.vdim) {
        const float z = gate[h * d.vdim + c], sg = sigmoid_f(z);
        out[row * ldo + h * d.vdim + c] = (AT)(o[i] * inv * w.norm[c] * (d.sigmoid_gate ? sg : z * sg));
      }
    }
  }
  if (r.last[row] - row < d.taps) {
    const int kw = d.kv_heads * d.dim, C = d.channels();
    float* ring = hist + r.slot[row] * h_elems + (int64_t)(r.pos[row] % d.taps) * C;
    for (int c = threadIdx.x; c < kw; c += 256) { ring[c] = p[in.oq + c]; ring[kw + c] = p[in.ok + c]; }
    for (int c = threadIdx.x; c < vw; c += 256) ring[2 * kw + c] = p[in.ov + c];
  }
}

// ------------------------------------------------------------------------------------------
// decode: one token of each entry, one work-group per (head, row): low-rank seconds, convolutions, unit norms, decay, the state
// update, output norm and gate.  The state is requested first and sits in registers while the rest is made.
// ------------------------------------------------------------------------------------------
template <typename AT, int RPT>
__global__ __launch_bounds__(1024) void delta_single_kernel(const DeltaDims d, const DeltaIn in, const DeltaW w, const uint16_t* a2, const int lda2, const uint16_t* g2, const int ldg2,
                                                            float* state, const int64_t s_elems, float* hist, const int64_t h_elems, const StepRows r, AT* out, const int64_t ldo, const int ct_log)
{
  __shared__ float sq[256], sk[256], sg[256], sv[256], sgate[256], so[256];
  __shared__ f32x4 su[32];
  __shared__ float sra[512], srg[512];
  __shared__ float red[2][16][128];
  __shared__ float sc[1];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int pos = r.pos[row], slot = r.slot[row];
  const int hg = d.heads / d.kv_heads, g = h / hg, kw = d.kv_heads * d.dim, C = d.channels();
  // a thread holds four consecutive columns of RPT rows; CT threads a row, RG rows side by side
  const int CT = 1 << ct_log, CP = CT * 4, RG = 1024 >> ct_log, ct = tid & (CT - 1), rg = tid >> ct_log;
  const int dvp = d.vdim_p();
  float* Sg = state + slot * s_elems + (int64_t)h * d.dim * dvp;
  f32x4 S[RPT];
  auto load_state = [&](int c0) {
#pragma unroll
    for (int j = 0; j < RPT; j++) {
      const int rr = rg + j * RG;
      S[j] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
      if (pos > 0 && rr < d.dim && c0 + ct * 4 < dvp) S[j] = *reinterpret_cast<const f32x4*>(Sg + (unsigned)(rr * dvp + c0 + ct * 4));
    }
  };
  load_state(0);
  const float* p = in.proj + row * in.ldp;
  float* ring = hist + slot * h_elems;
  float* ring_now = ring + (int64_t)(pos % d.taps) * C;
  for (int i = tid; i < d.rank_a; i += 1024) sra[i] = p[in.oa + i];
  for (int i = tid; i < d.rank_g; i += 1024) srg[i] = p[in.og + i];
  if (d.rank_a || d.rank_g) __syncthreads();
  if (wave < 2) {                                        // q (wave 0) and k (wave 1): convolution and unit norm
    const int oc = wave ? in.ok : in.oq, hc = wave ? kw : 0;
    const float* cw = wave ? w.ck : w.cq;
    float v[4], s = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int c = lane + 64 * i, ch = g * d.dim + c;
      v[i] = c < d.dim ? conv_silu(p + oc, in.ldp, 0, pos, ring, C, hc, cw, d.taps, ch) : 0.0f;
      s = fmaf(v[i], v[i], s);
    }
    const float nrm = (wave ? 1.0f : rsqrtf((float)d.dim)) / sqrtf(wave_total(s) + 1e-6f);
    float* dst = wave ? sk : sq;
#pragma unroll
    for (int i = 0; i < 4; i++) dst[lane + 64 * i] = v[i] * nrm;
    if (h % hg == 0) for (int c = lane; c < d.dim; c += 64) ring_now[hc + g * d.dim + c] = p[oc + g * d.dim + c];
  } else if (wave < 4) {                                 // v
    for (int c = tid - 128; c < d.vdim; c += 128) {
      const int ch = h * d.vdim + c;
      sv[c] = conv_silu(p + in.ov, in.ldp, 0, pos, ring, C, 2 * kw, w.cv, d.taps, ch);
      ring_now[2 * kw + ch] = p[in.ov + ch];
    }
  } else {                                               // decay and gate, four lanes to a low-rank row
    const int quad = (tid - 256) >> 2, ql = tid & 3, nd = d.channel_decay ? d.dim : 1, rate_i = h;
    auto low = [&](const uint16_t* m, int ld, const float* v, int rank, int rw) {
      float s = 0.0f;
      const uint16_t* mr = m + (int64_t)rw * ld;
      for (int i = ql * 8; i < rank; i += 32) {          // (columns beyond the rank are zero in the matrix, the vector is guarded)
        const u32x4 u = *reinterpret_cast<const u32x4*>(mr + i);
#pragma unroll
        for (int j = 0; j < 4; j++) {
          if (i + 2 * j < rank) s = fmaf(bf16_lo(u[j]), v[i + 2 * j], s);
          if (i + 2 * j + 1 < rank) s = fmaf(bf16_hi(u[j]), v[i + 2 * j + 1], s);
        }
      }
      s += __shfl_xor(s, 1); s += __shfl_xor(s, 2);
      return s;
    };
    for (int i = quad; i < nd + d.vdim; i += 192) {
      if (i < nd) {
        const int c = h * nd + i;
        const float z = (d.rank_a ? low(a2, lda2, sra, d.rank_a, c) : p[in.oa + c]) + w.dt_bias[c];
        if (ql == 0) sg[i] = expf(w.rate[rate_i] * softplus_f(z));
      } else {
        const int c = h * d.vdim + i - nd;
        const float z = d.rank_g ? low(g2, ldg2, srg, d.rank_g, c) : p[in.og + c];
        if (ql == 0) { const float s = sigmoid_f(z); sgate[i - nd] = d.sigmoid_gate ? s : z * s; }
      }
    }
  }
  __syncthreads();
  if (wave == 0) {
    float s = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) s = fmaf(sq[lane + 64 * i], sk[lane + 64 * i], s);
    s = wave_total(s);
    if (lane == 0) sc[0] = s;
  }
  const float beta = sigmoid_f(p[in.ob + h]);
  for (int c0 = 0; c0 < d.vdim; c0 += CP) {
    if (c0) load_state(c0);
    f32x4 ks = {0.0f, 0.0f, 0.0f, 0.0f}, qd = ks;
#pragma unroll
    for (int j = 0; j < RPT; j++) {
      const int rr = rg + j * RG;
      if (rr >= d.dim) continue;
      const float gr = sg[d.channel_decay ? rr : 0], kr = sk[rr], qr = sq[rr];
#pragma unroll
      for (int i = 0; i < 4; i++) { S[j][i] *= gr; ks[i] = fmaf(S[j][i], kr, ks[i]); qd[i] = fmaf(S[j][i], qr, qd[i]); }
    }
    for (int m = CT; m < 64; m <<= 1) {
#pragma unroll
      for (int i = 0; i < 4; i++) { ks[i] += __shfl_xor(ks[i], m); qd[i] += __shfl_xor(qd[i], m); }
    }
    if (lane < CT) { *reinterpret_cast<f32x4*>(&red[0][wave][ct * 4]) = ks; *reinterpret_cast<f32x4*>(&red[1][wave][ct * 4]) = qd; }
    __syncthreads();
    if (tid < 2 * CP) {
      const int which = tid >= CP, c = which ? tid - CP : tid;
      float a = 0.0f;
#pragma unroll
      for (int i = 0; i < 16; i++) a += red[which][i][c];
      if (which) { if (c0 + c < d.vdim) so[c0 + c] = a; }
      else reinterpret_cast<float*>(su)[c] = c0 + c < d.vdim ? beta * (sv[c0 + c] - a) : 0.0f;
    }
    __syncthreads();
    const f32x4 u = su[ct];
    if (tid < CP && c0 + tid < d.vdim) so[c0 + tid] = fmaf(sc[0], reinterpret_cast<float*>(su)[tid], so[c0 + tid]);
#pragma unroll
    for (int j = 0; j < RPT; j++) {
      const int rr = rg + j * RG;
      if (rr >= d.dim || c0 + ct * 4 >= dvp) continue;
      const float kr = sk[rr];
#pragma unroll
      for (int i = 0; i < 4; i++) S[j][i] = fmaf(kr, u[i], S[j][i]);
      *reinterpret_cast<f32x4*>(Sg + (unsigned)(rr * dvp + c0 + ct * 4)) = S[j];
    }
  }
  __syncthreads();
  if (wave == 0) {
    float o[4], s = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; o[i] = c < d.vdim ? so[c] : 0.0f; s = fmaf(o[i], o[i], s); }
    const float inv = 1.0f / sqrtf(wave_total(s) / (float)d.vdim + d.eps);
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int c = lane + 64 * i;
      if (c < d.vdim) out[row * ldo + h * d.vdim + c] = (AT)(o[i] * inv * w.norm[c] * sgate[c]);
    }
  }
}

int delta_prep(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b)
{
  const int gw = d.channel_decay ? d.heads * d.dim : d.heads;
  const int units = d.kv_heads + (d.heads * d.vdim + 255) / 256 + (gw + 255) / 256 + 1;
  const dim3 grid((r.n_rows + PREP_ROWS - 1) / PREP_ROWS, (units + 3) / 4);
  if (d.taps == 4) hipLaunchKernelGGL(delta_prep_kernel<4>, grid, dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b);
  else hipLaunchKernelGGL(delta_prep_kernel<0>, grid, dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int delta_scan(const DeltaDims& d, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b)
{
  const dim3 grid((d.vdim + 15) / 16, d.heads, r.n_ent), blk(256);
  auto s = ctx().stream;
#define SCAN(RPL) do { if (d.channel_decay) hipLaunchKernelGGL((delta_scan_kernel<RPL, true>), grid, blk, 0, s, d, st.S, st.s_elems, r, b); \
                       else hipLaunchKernelGGL((delta_scan_kernel<RPL, false>), grid, blk, 0, s, d, st.S, st.s_elems, r, b); } while (0)
  if (d.dim <= 64) SCAN(4); else if (d.dim <= 128) SCAN(8); else SCAN(16);
#undef SCAN
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int delta_chunked(const DeltaDims& d, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b, const int32_t* chunks, int n_chunks, const int32_t* chunk0)
{
  auto s = ctx().stream;
  const size_t lds = (size_t)(d.channel_decay ? 3 : 2) * CHUNK * (((d.dim + 15) & ~15) + 4) * 4;
  const dim3 g1(n_chunks, d.heads), g2((d.vdim + 15) / 16 * d.heads, r.n_ent), blk(256);
  if (d.channel_decay) hipLaunchKernelGGL(delta_chunk_kernel<true>, g1, blk, lds, s, d, r, b, chunks);
  else hipLaunchKernelGGL(delta_chunk_kernel<false>, g1, blk, lds, s, d, r, b, chunks);
#define WALK_V(NW, N, CH) do { if (d.dim % 4 == 0) hipLaunchKernelGGL((delta_walk_kernel<NW, N, CH, true>), g2, dim3(64 * (NW + 1)), 0, s, d, st.S, st.s_elems, r, b, chunk0); \
                               else hipLaunchKernelGGL((delta_walk_kernel<NW, N, CH, false>), g2, dim3(64 * (NW + 1)), 0, s, d, st.S, st.s_elems, r, b, chunk0); } while (0)
#define WALK(NW, N) do { if (d.channel_decay) WALK_V(NW, N, true); else WALK_V(NW, N, false); } while (0)
  if (d.dim <= 64) WALK(4, 1); else if (d.dim <= 128) WALK(4, 2); else WALK(8, 2);
#undef WALK
#undef WALK_V
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int delta_finish(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b, int act_t, void* out, int64_t ldo)
{
  if (act_t == ACT_T_BF16) hipLaunchKernelGGL(delta_finish_kernel<bf16_t>, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b, (bf16_t*)out, ldo);
  else hipLaunchKernelGGL(delta_finish_kernel<float>, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b, (float*)out, ldo);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int delta_single(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::StateRun& st, const StepRows& r, int act_t, void* out, int64_t ldo)
{
  const int ct_log = d.vdim > 64 ? 5 : d.vdim > 32 ? 4 : 3, rgs = 1024 >> ct_log, rpt = (d.dim + rgs - 1) / rgs;
  const dim3 grid(d.heads, r.n_rows), blk(1024);
  const uint16_t* a2 = w.a2 ? (const uint16_t*)w.a2->data : nullptr; const uint16_t* g2 = w.g2 ? (const uint16_t*)w.g2->data : nullptr;
  const int la = w.a2 ? (int)w.a2->ld : 0, lg = w.g2 ? (int)w.g2->ld : 0;
  auto s = ctx().stream;
#define SINGLE(AT, N) hipLaunchKernelGGL((delta_single_kernel<AT, N>), grid, blk, 0, s, d, in, w, a2, la, g2, lg, st.S, st.s_elems, st.hist, st.h_elems, r, (AT*)out, ldo, ct_log)
#define SINGLE_N(AT) do { if (rpt <= 2) SINGLE(AT, 2); else if (rpt <= 4) SINGLE(AT, 4); else SINGLE(AT, 8); } while (0)
  if (act_t == ACT_T_BF16) SINGLE_N(bf16_t); else SINGLE_N(float);
#undef SINGLE_N
#undef SINGLE
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

}  // namespace cai
