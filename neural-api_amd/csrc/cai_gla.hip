// Linear attention in which the forget gate also decides what is written: prompt kernels (chunks, the walk over them, the output norm)
// and a decode kernel.
//
// Per head a float state S [dim][vdim] (rows padded to four columns, the padding stays zero); one token does
//     f = l + (1 - l) sigmoid(. + bias),   S <- diag(f) S + (1 - f) v^T,   o = S^T q,   q = silu(.),
// with gates f and lower bounds l per head and channel; then an RMS norm over each head's o.  What is written, 1 - f, is made as
// (1 - l) sigmoid(-(. + bias)), so that a gate close to one costs it no accuracy.  Everything is 32-bit, the products of prompts run on
// the float matrix cores.
#include "cai_recurrent.hpp"

#include <algorithm>

namespace cai {

constexpr int GCHUNK = DELTA_CHUNK;

// ------------------------------------------------------------------------------------------
// prompt pass 1, everything of a chunk of 16 tokens that does not need the state (k = 1 - f, P_t the product of the chunk's gates up to
// t, all inclusive):
//   qt_t = P_t q_t,   kz_s = k_s f_s+1 .. f_15,   the chunk's whole decay P_15,   A_ts = q_t . (f_s+1 .. f_t k_s) for s <= t.
// Gates enter as running products only, never as quotients or differences of logarithms.
// ------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void gla_chunk_kernel(const GlaDims d, const GlaIn in, const GlaW w, const StepRows r, const DeltaBuf b, const int32_t* chunks)
{
  extern __shared__ float lds[];
  const int tid = threadIdx.x, h = blockIdx.y;
  const int32_t* en = r.ent + 4 * chunks[2 * blockIdx.x];
  const int t0 = chunks[2 * blockIdx.x + 1], nt = min(GCHUNK, en[2] - t0);
  const int64_t row0 = en[1] + t0;
  const int gw = d.heads * d.dim, dp = (d.dim + 15) & ~15, DS = dp + 4;
  float *sk = lds, *sq = lds + GCHUNK * DS, *sf = lds + 2 * GCHUNK * DS;
  for (int e = tid; e < GCHUNK * dp; e += 256) {
    const int t = e / dp, c = e - t * dp;
    const bool ok = t < nt && c < d.dim;
    const int cc = h * d.dim + (ok ? c : 0);
    const float* p = in.proj + (row0 + (ok ? t : 0)) * in.ldp;
    const float q = p[in.oq + cc], z = p[in.of + cc] + w.bias[cc], l = w.lower[cc];
    sq[t * DS + c] = ok ? q * sigmoid_f(q) : 0.0f;
    sk[t * DS + c] = ok ? (1.0f - l) * sigmoid_f(-z) : 0.0f;
    sf[t * DS + c] = ok ? fmaf(1.0f - l, sigmoid_f(z), l) : 1.0f;
  }
  __syncthreads();
  // thread (s, 16 channel lanes): what token s wrote, as the later tokens find it
  {
    const int s = tid >> 4, cl = tid & 15;
    float o[GCHUNK];
#pragma unroll
    for (int t = 0; t < GCHUNK; t++) o[t] = 0.0f;
    for (int c = cl; c < dp; c += 16) {
      float e = sk[s * DS + c];
#pragma unroll
      for (int t = 0; t < GCHUNK; t++) {
        e = t > s ? e * sf[t * DS + c] : e;
        o[t] = fmaf(sq[t * DS + c], e, o[t]);
      }
    }
#pragma unroll
    for (int t = 0; t < GCHUNK; t++) {
      const float y = row16_total(o[t]);
      if (cl == 0 && t < nt) b.qk[((row0 + t) * d.heads + h) * GCHUNK + s] = t >= s ? y : 0.0f;
    }
  }
  for (int c = tid; c < d.dim; c += 256) {
    float z = 1.0f, p = 1.0f, f[GCHUNK];
#pragma unroll
    for (int t = GCHUNK - 1; t >= 0; t--) {
      f[t] = sf[t * DS + c];
      if (t < nt) b.g[(row0 + t) * gw + h * d.dim + c] = sk[t * DS + c] * z;
      z *= f[t];
    }
#pragma unroll
    for (int t = 0; t < GCHUNK; t++) {
      p *= f[t];
      if (t < nt) b.qt[(row0 + t) * gw + h * d.dim + c] = sq[t * DS + c] * p;
    }
    b.gt[(int64_t)blockIdx.x * gw + h * d.dim + c] = p;
  }
}

// ------------------------------------------------------------------------------------------
// prompt pass 2: the walk, one work-group per (16 value columns, head, entry).  With S the state before the chunk,
//     o_t = S^T qt_t + sum_{s<=t} A_ts v_s,      S <- diag(P_15) S + sum_s kz_s v_s^T.
// Waves 0 .. NW - 1 hold the state - wave w the channels of tiles w TPW .. as matrix-core result registers, which are at the same time
// the right operand of the read-out - and wave NW finishes the chunk's rows of o while the others are a chunk further.  One barrier a
// chunk; the read-out's partial sums live in LDS for two chunks.
// ------------------------------------------------------------------------------------------
template <int NW, int TPW, bool VEC>       // VEC: the width of a head is a multiple of four
__global__ __launch_bounds__(64 * (NW + 1)) void gla_walk_kernel(const GlaDims d, const GlaIn in, float* state, const int64_t s_elems, const StepRows r, const DeltaBuf b, const int32_t* chunk0)
{
  __shared__ f32x4 po[2][NW][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), fr = lane & 15, fg = lane >> 4;
  // consecutive work-groups go to different XCDs; the column slices of a head read the same chunk data, so with heads in whole
  // eights every head stays on one XCD (and in its L2)
  const int slices = (d.vdim + 15) / 16;
  const int h = d.heads % 8 == 0 ? (blockIdx.x & 7) + 8 * ((blockIdx.x >> 3) / slices) : blockIdx.x / slices;
  const int col = (d.heads % 8 == 0 ? (blockIdx.x >> 3) % slices : blockIdx.x % slices) * 16 + fr;
  const int32_t* en = r.ent + 4 * blockIdx.y;
  const int slot = en[0], row0 = en[1], n = en[2], pos0 = en[3], ch0 = chunk0[blockIdx.y];
  const int vw = d.heads * d.vdim, gw = d.heads * d.dim, dvp = d.vdim_p(), nc = (n + GCHUNK - 1) / GCHUNK;
  // (rows past the portion's end are other rows, or the slack behind the last one; they and columns past the width are replaced by zeros
  // at use, or meet zeros)
  const int64_t lv = (int64_t)fg * 4 * in.ldp + in.ov + h * d.vdim + min(col, d.vdim - 1);
  auto fetch_v = [&](int c, float* v) {
    const float* p = in.proj + (int64_t)(row0 + min(c, nc - 1) * GCHUNK) * in.ldp + lv;
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = p[i * in.ldp];
  };
  if (wave == NW) {
    struct Out { float v[4]; f32x4 a; };
    auto fetch = [&](int c, Out& x) {
      fetch_v(c, x.v);
      x.a = *reinterpret_cast<const f32x4*>(b.qk + ((int64_t)(row0 + min(c, nc - 1) * GCHUNK + fr) * d.heads + h) * GCHUNK + fg * 4);
    };
    auto chunk = [&](int c, const Out& x) {
      __syncthreads();
      const int nt = n - c * GCHUNK;
      if (nt <= 0) return;
      f32x4 o = po[c & 1][0][lane];
#pragma unroll
      for (int v = 1; v < NW; v++) o += po[c & 1][v][lane];
#pragma unroll
      for (int i = 0; i < 4; i++) o = __builtin_amdgcn_mfma_f32_16x16x4f32(fr < nt ? x.a[i] : 0.0f, fg * 4 + i < nt ? x.v[i] : 0.0f, o, 0, 0, 0);
      float* ob = b.o + (int64_t)(row0 + c * GCHUNK + fg * 4) * vw + h * d.vdim + col;
#pragma unroll
      for (int i = 0; i < 4; i++) if (fg * 4 + i < nt && col < d.vdim) ob[(int64_t)i * vw] = o[i];
    };
    Out xa, xb, xc;
    fetch(0, xa); fetch(1, xb);
    for (int c = 0; c < nc; c += 3) {      // (as many barriers as the other waves meet)
      fetch(c + 2, xc); chunk(c, xa);
      fetch(c + 3, xa); chunk(c + 1, xb);
      fetch(c + 4, xb); chunk(c + 2, xc);
    }
    return;
  }
  float* Sg = state + slot * s_elems + (int64_t)h * d.dim * dvp;
  f32x4 S[TPW];
  bool ok4[TPW][VEC ? 1 : 4], ok1[TPW];
  unsigned l4[TPW], lq[TPW], lk[TPW];
#pragma unroll
  for (int j = 0; j < TPW; j++) {
    const int c4 = (wave * TPW + j) * 16 + fg * 4, c1 = (wave * TPW + j) * 16 + fr;
    ok1[j] = c1 < d.dim;
#pragma unroll
    for (int i = 0; i < (VEC ? 1 : 4); i++) ok4[j][i] = c4 + i < d.dim;
    l4[j] = c4 < d.dim ? c4 : 0;
    lq[j] = fr * gw + l4[j];
    lk[j] = fg * 4 * gw + (ok1[j] ? c1 : 0);
#pragma unroll
    for (int i = 0; i < 4; i++) S[j][i] = pos0 > 0 && c4 + i < d.dim && col < d.vdim ? Sg[(int64_t)(c4 + i) * dvp + col] : 0.0f;
  }
  auto four = [&](const float* p, unsigned c) -> f32x4 {
    if (VEC) return *reinterpret_cast<const f32x4*>(p + c);
    return f32x4{p[c], p[c + 1], p[c + 2], p[c + 3]};                     // (may run into the next row: replaced at use)
  };
  // a chunk's inputs are requested two chunks ahead and stay as they come until they are used
  struct In { f32x4 q[TPW], k[TPW], tot[TPW]; float v[4]; };
  auto fetch = [&](int c, In& x) {
    const int cc = min(c, nc - 1);
    const int64_t rr = (int64_t)(row0 + cc * GCHUNK) * gw + h * d.dim;
    const float *qb = b.qt + rr, *kb = b.g + rr, *tb = b.gt + (int64_t)(ch0 + cc) * gw + h * d.dim;
#pragma unroll
    for (int j = 0; j < TPW; j++) {
      x.q[j] = four(qb, lq[j]); x.tot[j] = four(tb, l4[j]);
#pragma unroll
      for (int i = 0; i < 4; i++) x.k[j][i] = (kb + i * gw)[lk[j]];
    }
    fetch_v(c, x.v);
  };
  auto chunk = [&](int c, const In& x) {
    const int nt = n - c * GCHUNK;
    const bool rok = fr < nt;
    f32x4 o[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}};
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int j = 0; j < TPW; j++)
        o[(i * TPW + j) & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(rok && ok4[j][VEC ? 0 : i] ? x.q[j][i] : 0.0f, S[j][i], o[(i * TPW + j) & 1], 0, 0, 0);
    po[c & 1][wave][lane] = o[0] + o[1];
    __syncthreads();
    if (nt <= 0) return;
#pragma unroll
    for (int j = 0; j < TPW; j++)
#pragma unroll
      for (int i = 0; i < 4; i++) S[j][i] *= ok4[j][VEC ? 0 : i] ? x.tot[j][i] : 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
      for (int j = 0; j < TPW; j++) {
        const bool in_chunk = fg * 4 + i < nt;
        S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(in_chunk && ok1[j] ? x.k[j][i] : 0.0f, in_chunk ? x.v[i] : 0.0f, S[j], 0, 0, 0);
      }
  };
  In xa, xb, xc;
  fetch(0, xa); fetch(1, xb);
  for (int c = 0; c < nc; c += 3) {
    fetch(c + 2, xc);
    __builtin_amdgcn_sched_barrier(0);
    chunk(c, xa);
    fetch(c + 3, xa);
    __builtin_amdgcn_sched_barrier(0);
    chunk(c + 1, xb);
    fetch(c + 4, xb);
    __builtin_amdgcn_sched_barrier(0);
    chunk(c + 2, xc);
  }
#pragma unroll
  for (int j = 0; j < TPW; j++)
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int c = (wave * TPW + j) * 16 + fg * 4 + i;
      if (c < d.dim && col < dvp) Sg[(int64_t)c * dvp + col] = col < d.vdim ? S[j][i] : 0.0f;
    }
}

// prompt pass 3: per row and head RMS norm and gain, a wave a head
template <typename AT>
__global__ __launch_bounds__(256) void gla_finish_kernel(const GlaDims d, const GlaW w, const DeltaBuf b, AT* out, const int64_t ldo)
{
  const int64_t row = blockIdx.x;
  const int lane = threadIdx.x & 63, vw = d.heads * d.vdim;
  for (int h = threadIdx.x >> 6; h < d.heads; h += 4) {
    float o[4], s = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; o[i] = c < d.vdim ? b.o[row * vw + h * d.vdim + c] : 0.0f; s = fmaf(o[i], o[i], s); }
    const float inv = 1.0f / sqrtf(wave_total(s) / (float)d.vdim + d.eps);
#pragma unroll
    for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; if (c < d.vdim) out[row * ldo + h * d.vdim + c] = (AT)(o[i] * inv * w.norm[c]); }
  }
}

// ------------------------------------------------------------------------------------------
// decode: one token of each entry, one work-group per (head, row): gates, state update, read-out, norm.  The state is requested first and
// sits in registers while the rest is made.
// ------------------------------------------------------------------------------------------
template <typename AT, int RPT>
__global__ __launch_bounds__(512) void gla_single_kernel(const GlaDims d, const GlaIn in, const GlaW w, float* state, const int64_t s_elems, const StepRows r, AT* out, const int64_t ldo, const int ct_log)
{
  __shared__ float sq[256], sf[256], sk[256], so[256];
  __shared__ f32x4 red[8][32];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int pos = r.pos[row], slot = r.slot[row], dvp = d.vdim_p();
  // a thread holds four consecutive columns of RPT rows; CT threads a row, RG rows side by side
  const int CT = 1 << ct_log, CP = CT * 4, RG = 512 >> ct_log, ct = tid & (CT - 1), rg = tid >> ct_log;
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
  for (int c = tid; c < d.dim; c += 512) {
    const int cc = h * d.dim + c;
    const float q = p[in.oq + cc], z = p[in.of + cc] + w.bias[cc], l = w.lower[cc];
    sq[c] = q * sigmoid_f(q); sk[c] = (1.0f - l) * sigmoid_f(-z); sf[c] = fmaf(1.0f - l, sigmoid_f(z), l);
  }
  const float* vp = p + in.ov + h * d.vdim;
  __syncthreads();
  for (int c0 = 0; c0 < d.vdim; c0 += CP) {
    if (c0) load_state(c0);
    f32x4 v, o = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = c0 + ct * 4 + i < d.vdim ? vp[c0 + ct * 4 + i] : 0.0f;
#pragma unroll
    for (int j = 0; j < RPT; j++) {
      const int rr = rg + j * RG;
      if (rr >= d.dim || c0 + ct * 4 >= dvp) continue;
      const float f = sf[rr], k = sk[rr], q = sq[rr];
#pragma unroll
      for (int i = 0; i < 4; i++) { S[j][i] = fmaf(k, v[i], S[j][i] * f); o[i] = fmaf(S[j][i], q, o[i]); }
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
      so[c0 + tid] = s;
    }
  }
  __syncthreads();
  if (wave == 0) {
    float o[4], s = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; o[i] = c < d.vdim ? so[c] : 0.0f; s = fmaf(o[i], o[i], s); }
    const float inv = 1.0f / sqrtf(wave_total(s) / (float)d.vdim + d.eps);
#pragma unroll
    for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; if (c < d.vdim) out[row * ldo + h * d.vdim + c] = (AT)(o[i] * inv * w.norm[c]); }
  }
}

int gla_chunked(const GlaDims& d, const GlaIn& in, const GlaW& w, const SeqPool::StateRun& st, const StepRows& r, const DeltaBuf& b, const int32_t* chunks, int n_chunks, const int32_t* chunk0, int act_t, void* out, int64_t ldo)
{
  auto s = ctx().stream;
  const size_t lds = (size_t)3 * GCHUNK * (((d.dim + 15) & ~15) + 4) * 4;
  hipLaunchKernelGGL(gla_chunk_kernel, dim3(n_chunks, d.heads), dim3(256), lds, s, d, in, w, r, b, chunks);
  const dim3 grid((d.vdim + 15) / 16 * d.heads, r.n_ent);
#define WALK_V(NW, N, V) hipLaunchKernelGGL((gla_walk_kernel<NW, N, V>), grid, dim3(64 * (NW + 1)), 0, s, d, in, st.S, st.s_elems, r, b, chunk0)
#define WALK(NW, N) do { if (d.dim % 4 == 0) WALK_V(NW, N, true); else WALK_V(NW, N, false); } while (0)
  if (d.dim <= 64) WALK(4, 1); else if (d.dim <= 128) WALK(4, 2); else WALK(8, 2);
#undef WALK
#undef WALK_V
  if (act_t == ACT_T_BF16) hipLaunchKernelGGL(gla_finish_kernel<bf16_t>, dim3(r.n_rows), dim3(256), 0, s, d, w, b, (bf16_t*)out, ldo);
  else hipLaunchKernelGGL(gla_finish_kernel<float>, dim3(r.n_rows), dim3(256), 0, s, d, w, b, (float*)out, ldo);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int gla_single(const GlaDims& d, const GlaIn& in, const GlaW& w, const SeqPool::StateRun& st, const StepRows& r, int act_t, void* out, int64_t ldo)
{
  const int ct_log = d.vdim > 64 ? 5 : d.vdim > 32 ? 4 : 3, rgs = 512 >> ct_log, rpt = (d.dim + rgs - 1) / rgs;
#define SINGLE(AT, N) hipLaunchKernelGGL((gla_single_kernel<AT, N>), dim3(d.heads, r.n_rows), dim3(512), 0, ctx().stream, d, in, w, st.S, st.s_elems, r, (AT*)out, ldo, ct_log)
#define SINGLE_N(AT) do { if (rpt <= 2) SINGLE(AT, 2); else if (rpt <= 4) SINGLE(AT, 4); else if (rpt <= 8) SINGLE(AT, 8); else SINGLE(AT, 16); } while (0)
  if (act_t == ACT_T_BF16) SINGLE_N(bf16_t); else SINGLE_N(float);
#undef SINGLE_N
#undef SINGLE
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

}  // namespace cai
