// Gated delta rule with short convolutions: prompt kernels (convolution and unit norms, the scan, the gated output norm) and a
// one-launch decode kernel.
//
// Per head a float state S [dim][vdim] (rows padded to four columns, the padding stays zero); one token does  S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.
// With S' = diag(g) S the read-out is  o = S'^T q + (q . k) u, so both products with S' are taken together and the second
// reduction is off the dependent chain.  Everything that touches the state is 32-bit.
//
// A sequence's last `taps` raw inputs of every convolved channel are kept in a ring (entry position mod taps).  The ring has one
// entry more than a token looks back, so the entry the newest token takes is never one that the same step still reads.
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
__device__ __forceinline__ float conv_silu(const float* cur, int64_t ldp, int back, int pos, const float* ring, int channels, int hc, const float* w, int taps, int c)
{
  float s = w[c * taps + taps - 1] * cur[c];
  for (int j = 1; j < taps; j++) {
    float x = 0.0f;
    if (j <= back) x = cur[c - (int64_t)j * ldp];
    else if (j <= pos) x = ring[(int64_t)((pos - j) % taps) * channels + hc + c];
    s = fmaf(w[c * taps + taps - 1 - j], x, s);
  }
  return s * sigmoid_f(s);
}

// ------------------------------------------------------------------------------------------
// prompt pass 1: q and k unit vectors (q scaled), v, decay (its logarithm for the chunked pass), write strength, q . k.
// A wave owns one unit - the q and k channels of a key head, 256 channels of v, 256 decays, the write strengths - over eight
// consecutive rows; the convolution slides over them, so each input is fetched once (TAPS = 4; other lengths look back per row).
// ------------------------------------------------------------------------------------------
constexpr int PREP_ROWS = 8;

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
  __device__ __forceinline__ float step(int i, float x)
  {
    float s = w[i][TAPS - 1] * x;
#pragma unroll
    for (int j = 1; j < TAPS; j++) s = fmaf(w[i][TAPS - 1 - j], h[i][j - 1], s);
#pragma unroll
    for (int j = TAPS - 2; j > 0; j--) h[i][j] = h[i][j - 1];
    h[i][0] = x;
    return s * sigmoid_f(s);
  }
};

template <int TAPS>
__global__ __launch_bounds__(256) void delta_prep_kernel(const DeltaDims d, const DeltaIn in, const DeltaW w, const float* hist, const int64_t h_elems, const StepRows r, const DeltaBuf b, const int log_decay)
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
        const float l = rate * softplus_f(z + bias);
        b.g[(int64_t)row * gw + c] = log_decay ? l : expf(l);
      }
    }
    return;
  }
  if (unit == ng)
    for (int row = r0; row < r1; row++)
      for (int h = lane; h < d.heads; h += 64) b.beta[(int64_t)row * bw + h] = sigmoid_f(in.proj[row * in.ldp + in.ob + h]);
}

// ------------------------------------------------------------------------------------------
// prompt pass 2: the scan.  A wave owns four columns of one head's state: 16 lanes a column, RPL rows a lane (rows
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

int delta_prep(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::DeltaRun& st, const StepRows& r, const DeltaBuf& b, bool log_decay)
{
  const int gw = d.channel_decay ? d.heads * d.dim : d.heads;
  const int units = d.kv_heads + (d.heads * d.vdim + 255) / 256 + (gw + 255) / 256 + 1;
  const dim3 grid((r.n_rows + PREP_ROWS - 1) / PREP_ROWS, (units + 3) / 4);
  if (d.taps == 4) hipLaunchKernelGGL(delta_prep_kernel<4>, grid, dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b, (int)log_decay);
  else hipLaunchKernelGGL(delta_prep_kernel<0>, grid, dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b, (int)log_decay);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int delta_scan(const DeltaDims& d, const SeqPool::DeltaRun& st, const StepRows& r, const DeltaBuf& b)
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

int delta_finish(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::DeltaRun& st, const StepRows& r, const DeltaBuf& b, int act_t, void* out, int64_t ldo)
{
  if (act_t == ACT_T_BF16) hipLaunchKernelGGL(delta_finish_kernel<bf16_t>, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b, (bf16_t*)out, ldo);
  else hipLaunchKernelGGL(delta_finish_kernel<float>, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, in, w, st.hist, st.h_elems, r, b, (float*)out, ldo);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int delta_single(const DeltaDims& d, const DeltaIn& in, const DeltaW& w, const SeqPool::DeltaRun& st, const StepRows& r, int act_t, void* out, int64_t ldo)
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
