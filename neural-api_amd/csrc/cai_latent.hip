// Latent attention over pages: per token one normed latent, shared by all heads' keys and values, and one key part that turns with the
// position are cached.  With k_h = A_h c and v_h = B_h c (c the latent),
//     score = (q_h . A_h c + turned parts) scale = ((A_h^T q_h) . c + ...) scale,      o_h = sum_j w_j B_h c_j = B_h (sum_j w_j c_j).
//
// Two forms.  The row form (decoded tokens, short portions, the all-32-bit mode) takes queries into the latent's space, meets the cached
// rows as they are and sends the sums of latents through B_h: a cached row is read once for a group of heads, and nothing is made of
// it.  The expanded form (prompts) makes keys and values of all of an entry's positions with one product and runs the matrix-core
// attention over them, whose products over a head's own width are a fraction of those over the latent's.
// Latents' norms, turning, scores, soft-max and weights are 32-bit in both.
#include "cai_layered.hpp"
#include "cai_recurrent.hpp"

#include <algorithm>

namespace cai {

constexpr int LSLICE = PAGE_TOKENS;        // keys per work-group of the row form: a page

template <typename T> __device__ __forceinline__ void load_eight(const T* p, float* v)
{
  if constexpr (sizeof(T) == 2) {
    const u32x4 u = *reinterpret_cast<const u32x4*>(p);
#pragma unroll
    for (int j = 0; j < 4; j++) { v[2 * j] = bf16_lo(u[j]); v[2 * j + 1] = bf16_hi(u[j]); }
  } else {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), c = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int j = 0; j < 4; j++) { v[j] = a[j]; v[4 + j] = c[j]; }
  }
}
template <typename T> __device__ __forceinline__ T* latent_page(const KvView& kv, int slot, int page)
{
  return reinterpret_cast<T*>(kv.base) + (int64_t)kv.table[slot * kv.ring + page % kv.ring] * kv.page_elems;
}

// element c of a turned part x at a position: neighbours 2i, 2i + 1 turn together.  The angle is reduced in turns with double precision
// before sine and cosine.
__device__ __forceinline__ float turned(const LatentDims& d, const float* x, int c, int pos)
{
  if (c >= d.rot) return x[c];
  const double t = (double)pos * d.turns[c >> 1];
  float sn, cs;
  sincospif((float)(2.0 * (t - rint(t))), &sn, &cs);
  const float v = c & 1 ? x[c] * cs + x[c - 1] * sn : x[c] * cs - x[c + 1] * sn;
  return v * d.amp;
}

// by a work-group of 256: the normed latent and the turned part of a row into its page; red: LDS for 4 floats
template <typename T> __device__ __forceinline__ void append_row(const LatentDims& d, const KvView& kv, const LatentIn& in, const StepRows& r, int row, float* red)
{
  const int tid = threadIdx.x, pos = r.pos[row];
  const float* p = in.proj + row * in.ldp + in.okv;
  T* dst = latent_page<T>(kv, r.slot[row], pos / PAGE_TOKENS) + (int64_t)(pos % PAGE_TOKENS) * d.lat_p();
  float s = 0.0f;
  for (int c = tid; c < d.kv_rank; c += 256) s = fmaf(p[c], p[c], s);
  s = wave_total(s);
  if ((tid & 63) == 0) red[tid >> 6] = s;
  __syncthreads();
  const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)d.kv_rank + d.eps);
  const int lc = d.lat_c();
  for (int c = tid; c < d.lat_p(); c += 256)
    dst[c] = (T)(c < lc ? (c < d.kv_rank ? p[c] * inv * in.kvn[c] : 0.0f) : c - lc < d.rot_dim ? turned(d, p + d.kv_rank, c - lc, pos) : 0.0f);
}

template <typename T>
__global__ __launch_bounds__(256) void latent_append_kernel(const LatentDims d, const KvView kv, const LatentIn in, const StepRows r, T* qlat, const int64_t ldl)
{
  __shared__ float red[4], red2[4];
  const int row = blockIdx.x, tid = threadIdx.x;
  append_row<T>(d, kv, in, r, row, red);
  if (!qlat) return;
  const float* p = in.proj + row * in.ldp + in.oq;
  float s = 0.0f;
  for (int c = tid; c < d.q_rank; c += 256) s = fmaf(p[c], p[c], s);
  s = wave_total(s);
  if ((tid & 63) == 0) red2[tid >> 6] = s;
  __syncthreads();
  const float inv = 1.0f / sqrtf((red2[0] + red2[1] + red2[2] + red2[3]) / (float)d.q_rank + d.eps);
  for (int c = tid; c < ldl; c += 256) qlat[row * ldl + c] = (T)(c < d.q_rank ? p[c] * inv * in.qn[c] : 0.0f);
}

// ------------------------------------------------------------------------------------------
// Row form, first launch: A_h^T q_h and the turned part.  blockIdx: x head, y 128 columns of the latent, z NB rows; sixteen lanes take
// eight columns each, sixteen groups of them share the head's width.  APPEND: one head more, whose work-groups (y = 0) bring the rows'
// latents into the pages (T: the pages' type).
// ------------------------------------------------------------------------------------------
template <typename T, int NB, bool APPEND>
__global__ __launch_bounds__(256) void latent_absorb_kernel(const LatentDims d, const KvView kv, const LatentIn in, const uint16_t* up, const int ldu, const StepRows r, const int32_t* rows, const int n_rows, float* qabs)
{
  __shared__ float sq[NB][256], part[4][NB][128], red[4];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), h = blockIdx.x, z0 = blockIdx.z * NB;
  auto row_of = [&](int b) { const int z = min(z0 + b, n_rows - 1); return rows ? rows[z] : z; };
  if (APPEND && h == d.heads) {
    if (blockIdx.y == 0)
      for (int b = 0; b < NB && z0 + b < n_rows; b++) {
        if (b) __syncthreads();
        append_row<T>(d, kv, in, r, row_of(b), red);
      }
    return;
  }
  const int dq = d.dim + d.rot_dim, l16 = tid & 15, dg = tid >> 4, c0 = blockIdx.y * 128 + l16 * 8;
#pragma unroll
  for (int b = 0; b < NB; b++) {
    const float* q = in.qraw + (int64_t)row_of(b) * in.ldq + h * dq;
    for (int c = tid; c < d.dim; c += 256) sq[b][c] = q[c];
  }
  __syncthreads();
  float acc[NB][8];
#pragma unroll
  for (int b = 0; b < NB; b++)
#pragma unroll
    for (int i = 0; i < 8; i++) acc[b][i] = 0.0f;
  if (c0 < ldu) {
    const uint16_t* m = up + (int64_t)h * d.head_e() * ldu + c0;
#pragma unroll 4
    for (int k = dg; k < d.dim; k += 16) {
      float v[8];
      load_eight(reinterpret_cast<const bf16_t*>(m + (int64_t)k * ldu), v);
#pragma unroll
      for (int b = 0; b < NB; b++)
#pragma unroll
        for (int i = 0; i < 8; i++) acc[b][i] = fmaf(sq[b][k], v[i], acc[b][i]);
    }
  }
#pragma unroll
  for (int b = 0; b < NB; b++)
#pragma unroll
    for (int i = 0; i < 8; i++) {
      acc[b][i] += __shfl_xor(acc[b][i], 16); acc[b][i] += __shfl_xor(acc[b][i], 32);
      if (lane < 16) part[wave][b][lane * 8 + i] = acc[b][i];
    }
  __syncthreads();
  const int lc = d.lat_c(), lp = d.lat_p();
  for (int e = tid; e < NB * 128; e += 256) {
    const int b = e >> 7, c = blockIdx.y * 128 + (e & 127);
    if (z0 + b >= n_rows || c >= lc) continue;
    qabs[((int64_t)(z0 + b) * d.heads + h) * lp + c] = c < d.kv_rank ? part[0][b][e & 127] + part[1][b][e & 127] + part[2][b][e & 127] + part[3][b][e & 127] : 0.0f;
  }
  if (blockIdx.y) return;
  for (int e = tid; e < NB * (lp - lc); e += 256) {
    const int b = e / (lp - lc), c = e % (lp - lc);
    if (z0 + b >= n_rows) continue;
    const int row = row_of(b);
    qabs[((int64_t)(z0 + b) * d.heads + h) * lp + lc + c] = c < d.rot_dim ? turned(d, in.qraw + (int64_t)row * in.ldq + h * dq + d.dim, c, r.pos[row]) : 0.0f;
  }
}

// ------------------------------------------------------------------------------------------
// Row form, second launch: blockIdx x = page of keys, y = HT heads, z = row.  Sixteen lanes a key for the scores, eight columns a lane and
// turn; then eight columns a lane and sixteen keys for the sums.  part: per (row, head, slice) lat_c sums, the maximum, the normaliser.
// ------------------------------------------------------------------------------------------
template <typename T, int HT>
__global__ __launch_bounds__(256) void latent_rows_kernel(const LatentDims d, const KvView kv, const StepRows r, const int32_t* rows, const float* qabs, float* part)
{
  extern __shared__ __align__(16) float sq[];            // [HT][lat_p]
  __shared__ float sc[HT][LSLICE];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), n_sl = gridDim.x;
  const int h0 = blockIdx.y * HT, nh = min(HT, d.heads - h0), z = blockIdx.z, row = rows ? rows[z] : z;
  const int pos = r.pos[row], k0 = blockIdx.x * LSLICE, nkeys = min(LSLICE, pos + 1 - k0);
  if (nkeys <= 0) return;                  // (part is only read up to the slices in use)
  const int lc = d.lat_c(), lp = d.lat_p();
  const T* page = latent_page<T>(kv, r.slot[row], blockIdx.x);
  const float* q = qabs + ((int64_t)z * d.heads + h0) * lp;
  for (int i = tid * 4; i < nh * lp; i += 1024) *reinterpret_cast<f32x4*>(sq + i) = *reinterpret_cast<const f32x4*>(q + i);
  for (int i = nh * lp + tid; i < HT * lp; i += 256) sq[i] = 0.0f;
  __syncthreads();
  {
    const int l16 = lane & 15, kb = wave * 4 + (lane >> 4);
    float s[HT][4];
#pragma unroll
    for (int hh = 0; hh < HT; hh++)
#pragma unroll
      for (int u = 0; u < 4; u++) s[hh][u] = 0.0f;
    const T* kp[4];
#pragma unroll
    for (int u = 0; u < 4; u++) kp[u] = page + (int64_t)min(kb + 16 * u, nkeys - 1) * lp;
#pragma unroll 2
    for (int c = l16 * 8; c < lp; c += 128) {
      float kx[4][8];
#pragma unroll
      for (int u = 0; u < 4; u++) load_eight<T>(kp[u] + c, kx[u]);
#pragma unroll
      for (int hh = 0; hh < HT; hh++) {
        float qv[8];
        *reinterpret_cast<f32x4*>(qv) = *reinterpret_cast<const f32x4*>(sq + hh * lp + c);
        *reinterpret_cast<f32x4*>(qv + 4) = *reinterpret_cast<const f32x4*>(sq + hh * lp + c + 4);
#pragma unroll
        for (int u = 0; u < 4; u++)
#pragma unroll
          for (int i = 0; i < 8; i++) s[hh][u] = fmaf(qv[i], kx[u][i], s[hh][u]);
      }
    }
#pragma unroll
    for (int hh = 0; hh < HT; hh++)
#pragma unroll
      for (int u = 0; u < 4; u++) {
        const float t = row16_total(s[hh][u]);
        if (l16 == 0) sc[hh][kb + 16 * u] = t * d.scale;
      }
  }
  __syncthreads();
  auto tail = [&](int hh) { return part + (((int64_t)z * d.heads + h0 + hh) * n_sl + blockIdx.x) * (lc + 2); };
  for (int hh = wave; hh < HT; hh += 4) {
    float v = hh < nh && lane < nkeys ? sc[hh][lane] : -INFINITY, m = v;
#pragma unroll
    for (int o = 32; o; o >>= 1) m = fmaxf(m, __shfl_xor(m, o));
    v = lane < nkeys && hh < nh ? expf(v - m) : 0.0f;
    sc[hh][lane] = v;
    const float s = wave_total(v);
    if (lane == 0 && hh < nh) { float* t = tail(hh) + lc; t[0] = m; t[1] = s; }
  }
  __syncthreads();
  const int kg = lane >> 4;
  for (int cb = wave * 16 + (lane & 15); cb - (lane & 15) < lc / 8; cb += 64) {    // (the lanes of a wave stay together for the sums)
    const int c = min(cb, lc / 8 - 1) * 8;
    float acc[HT][8];
#pragma unroll
    for (int hh = 0; hh < HT; hh++)
#pragma unroll
      for (int i = 0; i < 8; i++) acc[hh][i] = 0.0f;
#pragma unroll 4
    for (int k = kg; k < nkeys; k += 4) {
      float v[8];
      load_eight<T>(page + (int64_t)k * lp + c, v);
#pragma unroll
      for (int hh = 0; hh < HT; hh++) {
        const float p = sc[hh][k];
#pragma unroll
        for (int i = 0; i < 8; i++) acc[hh][i] = fmaf(p, v[i], acc[hh][i]);
      }
    }
#pragma unroll
    for (int hh = 0; hh < HT; hh++) {
      if (hh >= nh) break;
#pragma unroll
      for (int i = 0; i < 8; i++) { acc[hh][i] += __shfl_xor(acc[hh][i], 16); acc[hh][i] += __shfl_xor(acc[hh][i], 32); }
      if (kg == 0 && cb < lc / 8) {
        float* t = tail(hh) + c;           // (two floats more than eight per head: eight-byte aligned)
#pragma unroll
        for (int i = 0; i < 8; i += 2) *reinterpret_cast<float2*>(t + i) = make_float2(acc[hh][i], acc[hh][i + 1]);
      }
    }
  }
}

// Row form, third launch: the slices' sums of latents join, and B_h and the gate make the head's output.  blockIdx: x head, y row, z a part
// of the head's values; sixteen lanes a value.
template <typename AT>
__global__ __launch_bounds__(256) void latent_merge_kernel(const LatentDims d, const LatentIn in, const uint16_t* up, const int ldu, const StepRows r, const int32_t* rows, const int n_sl, const float* part, AT* out, const int64_t ldo)
{
  extern __shared__ __align__(16) float so[];            // [lat_c] up to whole 128s
  __shared__ float sm[4], sl[4], sw[256];
  const int h = blockIdx.x, z = blockIdx.y, row = rows ? rows[z] : z, pos = r.pos[row], tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lc = d.lat_c(), st = lc + 2, used = pos / LSLICE + 1;
  const float* p = part + ((int64_t)z * d.heads + h) * n_sl * st;
  float m = -INFINITY, l = 0.0f;
  for (int s = tid; s < used; s += 256) m = fmaxf(m, p[(int64_t)s * st + lc]);
#pragma unroll
  for (int o = 32; o; o >>= 1) m = fmaxf(m, __shfl_xor(m, o));
  if (lane == 0) sm[wave] = m;
  __syncthreads();
  m = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
  for (int s = tid; s < used; s += 256) l += p[(int64_t)s * st + lc + 1] * expf(p[(int64_t)s * st + lc] - m);
  l = wave_total(l);
  if (lane == 0) sl[wave] = l;
  for (int c0 = 0; c0 < lc; c0 += 512) {
    float a[2] = {0.0f, 0.0f};
    const int c[2] = {c0 + tid, c0 + tid + 256};
    for (int s0 = 0; s0 < used; s0 += 256) {             // a block of slice weights at a time
      const int ns = min(256, used - s0);
      __syncthreads();
      if (tid < ns) sw[tid] = expf(p[(int64_t)(s0 + tid) * st + lc] - m);
      __syncthreads();
      for (int s = 0; s < ns; s += 8) {
        float t[8][2];
#pragma unroll
        for (int k = 0; k < 8; k++)
#pragma unroll
          for (int u = 0; u < 2; u++) t[k][u] = p[(int64_t)(s0 + min(s + k, ns - 1)) * st + min(c[u], lc - 1)];
#pragma unroll
        for (int k = 0; k < 8; k++)
#pragma unroll
          for (int u = 0; u < 2; u++) a[u] = s + k < ns ? fmaf(t[k][u], sw[s + k], a[u]) : a[u];
      }
    }
    const float inv = 1.0f / (sl[0] + sl[1] + sl[2] + sl[3]);
#pragma unroll
    for (int u = 0; u < 2; u++) if (c[u] < ((lc + 127) & ~127)) so[c[u]] = c[u] < lc ? a[u] * inv : 0.0f;
  }
  __syncthreads();
  const int l16 = tid & 15, per = (d.vdim + gridDim.z - 1) / gridDim.z, v1 = min(d.vdim, (int)(blockIdx.z + 1) * per);
  const uint16_t* m0 = up + ((int64_t)h * d.head_e() + d.dim_e()) * ldu;
  for (int v0 = blockIdx.z * per; v0 < v1; v0 += 16) {
    const int v = v0 + (tid >> 4);
    const uint16_t* mr = m0 + (int64_t)min(v, v1 - 1) * ldu;
    float s = 0.0f;
    for (int c = l16 * 8; c < lc; c += 128) {
      float x[8];
      load_eight(reinterpret_cast<const bf16_t*>(mr + c), x);
      const f32x4 a = *reinterpret_cast<const f32x4*>(so + c), b = *reinterpret_cast<const f32x4*>(so + c + 4);
#pragma unroll
      for (int i = 0; i < 4; i++) { s = fmaf(x[i], a[i], s); s = fmaf(x[4 + i], b[i], s); }
    }
    s = row16_total(s);
    const int c = h * d.vdim + v;
    if (l16 == 0 && v < v1) out[row * ldo + c] = (AT)(s * sigmoid_f(in.proj[row * in.ldp + in.og + c]));
  }
}

// ------------------------------------------------------------------------------------------
// The expanded form's operands
// ------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void latent_queries_kernel(const LatentDims d, const LatentIn in, const StepRows r, bf16_t* qbuf)
{
  const int row = blockIdx.x, dq = d.dim + d.rot_dim, de = d.dim_e(), ke = d.key_e(), pos = r.pos[row];
  const float* q = in.qraw + (int64_t)row * in.ldq;
  bf16_t* o = qbuf + (int64_t)row * d.heads * ke;
  __shared__ float sn[256], cs[256];       // of the turned part's dimensions (rot_dim is a head's at most)
  for (int c = threadIdx.x; c < d.rot / 2; c += 256) {
    const double t = (double)pos * d.turns[c];
    float s, k;
    sincospif((float)(2.0 * (t - rint(t))), &s, &k);
    sn[c] = s; cs[c] = k;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < d.heads * ke; e += 256) {
    const int h = e / ke, c = e - h * ke;
    const float* x = q + h * dq;
    float v = 0.0f;
    if (c < de) { if (c < d.dim) v = x[c]; }
    else if (c - de < d.rot_dim) {
      const int t = c - de;
      x += d.dim;
      v = x[t];
      if (t < d.rot) v = (t & 1 ? v * cs[t >> 1] + x[t - 1] * sn[t >> 1] : v * cs[t >> 1] - x[t + 1] * sn[t >> 1]) * d.amp;
    }
    o[e] = (bf16_t)v;
  }
}

__global__ __launch_bounds__(256) void latent_gather_kernel(const LatentDims d, const KvView kv, const int32_t* pages, bf16_t* rows, const int64_t ldc)
{
  const bf16_t* page = latent_page<bf16_t>(kv, pages[2 * blockIdx.x], pages[2 * blockIdx.x + 1]);
  bf16_t* o = rows + (int64_t)blockIdx.x * PAGE_TOKENS * ldc;
  const int n = (int)ldc / 8, lc = d.lat_c(), lp = d.lat_p();
  for (int e = blockIdx.y * 256 + threadIdx.x; e < PAGE_TOKENS * n; e += gridDim.y * 256) {
    const int t = e / n, c = (e - t * n) * 8;
    *reinterpret_cast<u32x4*>(o + t * ldc + c) = c < lc ? *reinterpret_cast<const u32x4*>(page + t * lp + c) : u32x4{0, 0, 0, 0};
  }
}

int latent_append(const LatentDims& d, const KvView& kv, int act_t, const LatentIn& in, const StepRows& r, void* qlat, int64_t ldl)
{
  if (act_t == ACT_T_BF16) hipLaunchKernelGGL(latent_append_kernel<bf16_t>, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, kv, in, r, (bf16_t*)qlat, ldl);
  else hipLaunchKernelGGL(latent_append_kernel<float>, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, kv, in, r, (float*)qlat, ldl);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

static int latent_slices(const LatentDims& d, int reach) { return (std::min(d.span, reach) + LSLICE - 1) / LSLICE; }
static size_t latent_part_row(const LatentDims& d, int ns) { return (size_t)d.heads * ns * (d.lat_c() + 2); }
constexpr size_t LATENT_PART_FLOATS = 64 << 20;   // partial results of more rows than fit this are made in turns
size_t latent_part_floats(const LatentDims& d, int n_rows)
{
  const size_t one = latent_part_row(d, latent_slices(d, d.span));
  return std::max(one, std::min(LATENT_PART_FLOATS, (size_t)n_rows * one));
}

template <typename T, int NB>
static void run_absorb(const LatentDims& d, const KvView& kv, const LatentIn& in, const cai_qw_s* up, const StepRows& r, const int32_t* rows, int n_rows, bool append, float* qabs)
{
  const dim3 grid(d.heads + (append ? 1 : 0), (d.lat_c() + 127) / 128, (n_rows + NB - 1) / NB);
  if (append) hipLaunchKernelGGL((latent_absorb_kernel<T, NB, true>), grid, dim3(256), 0, ctx().stream, d, kv, in, (const uint16_t*)up->data, (int)up->ld, r, rows, n_rows, qabs);
  else hipLaunchKernelGGL((latent_absorb_kernel<T, NB, false>), grid, dim3(256), 0, ctx().stream, d, kv, in, (const uint16_t*)up->data, (int)up->ld, r, rows, n_rows, qabs);
}

template <typename T>
static int run_latent_rows(const LatentDims& d, const KvView& kv, const LatentIn& in, const cai_qw_s* up, const StepRows& r, const int32_t* rows, int n_rows, bool append, float* qabs,
                           float* part, size_t part_floats, T* out, int64_t ldo)
{
  auto st = ctx().stream;
  const int ns = latent_slices(d, r.reach), lp = d.lat_p();
  const size_t turn = std::min<size_t>(32768, part_floats / latent_part_row(d, ns));
  CAI_REQUIRE(turn >= 1, "latent attention: partial results of %d slices do not fit %zu floats", ns, part_floats);
  if (n_rows == 1) run_absorb<T, 1>(d, kv, in, up, r, rows, n_rows, append, qabs); else run_absorb<T, 4>(d, kv, in, up, r, rows, n_rows, append, qabs);
  const int ht = d.heads <= 4 || (int64_t)ns * ((d.heads + 7) / 8) * n_rows < ctx().n_cu ? 4 : 8;    // heads of a work-group
  for (int z0 = 0; z0 < n_rows; z0 += (int)turn) {
    const int m = std::min((int)turn, n_rows - z0);
    StepRows q = r; LatentIn a = in; const int32_t* list = rows; T* o = out;
    if (rows) list += z0;
    else { q.pos += z0; q.slot += z0; a.proj += z0 * in.ldp; o += (int64_t)z0 * ldo; }
    const float* qa = qabs + (int64_t)z0 * d.heads * lp;
    if (ht == 4) hipLaunchKernelGGL((latent_rows_kernel<T, 4>), dim3(ns, (d.heads + 3) / 4, m), dim3(256), (size_t)4 * lp * 4, st, d, kv, q, list, qa, part);
    else hipLaunchKernelGGL((latent_rows_kernel<T, 8>), dim3(ns, (d.heads + 7) / 8, m), dim3(256), (size_t)8 * lp * 4, st, d, kv, q, list, qa, part);
    int split = 1;                         // parts of a head's values, until every CU has two work-groups
    while (split < 8 && d.heads * m * split < 2 * ctx().n_cu && d.vdim / (2 * split) >= 16) split *= 2;
    hipLaunchKernelGGL(latent_merge_kernel<T>, dim3(d.heads, m, split), dim3(256), (size_t)pad_to(d.lat_c(), 128) * 4, st, d, a, (const uint16_t*)up->data, (int)up->ld, q, list, ns, part, o, ldo);
  }
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}
int latent_rows(const LatentDims& d, const KvView& kv, int act_t, const LatentIn& in, const cai_qw_s* up, const StepRows& r, const int32_t* rows, int n_rows, bool append, float* qabs,
                float* part, size_t part_floats, void* out, int64_t ldo)
{
  CAI_REQUIRE(d.dim <= 256 && d.lat_p() <= 1024, "latent attention: heads of %d, rows of %d", d.dim, d.lat_p());
  return act_t == ACT_T_BF16 ? run_latent_rows<bf16_t>(d, kv, in, up, r, rows, n_rows, append, qabs, part, part_floats, (bf16_t*)out, ldo)
                             : run_latent_rows<float>(d, kv, in, up, r, rows, n_rows, append, qabs, part, part_floats, (float*)out, ldo);
}

bool latent_expand_ok(const LatentDims& d, int act_t) { return act_t == ACT_T_BF16 && d.key_e() <= 256 && d.vdim_e() <= 256; }

int latent_queries(const LatentDims& d, const LatentIn& in, const StepRows& r, void* qbuf)
{
  hipLaunchKernelGGL(latent_queries_kernel, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, in, r, (bf16_t*)qbuf);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}
int latent_gather(const LatentDims& d, const KvView& kv, const int32_t* pages, int n_pages, void* rows, int64_t ldc)
{
  hipLaunchKernelGGL(latent_gather_kernel, dim3(n_pages, 4), dim3(256), 0, ctx().stream, d, kv, pages, (bf16_t*)rows, ldc);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

}  // namespace cai
