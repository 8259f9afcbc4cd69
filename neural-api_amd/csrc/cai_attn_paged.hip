// Grouped-query attention over a paged key/value pool, in a sliding window or in fixed blocks of positions: key and value widths of
// their own, optional RMS norm of queries and keys (per head or over all heads at once), optional rotation of the first dimensions of
// a head, optional growth of the queries with the position, an explicit score scale, an optional sigmoid gate on the heads' outputs.
// The weights are a soft-max over the keys (a sink, a number without a key, may join its normaliser) or, each key for itself, a sigmoid of the score with a logarithmic loss over the distance.
// A run may read the pages that an earlier run has filled.
//
// Two forms: one work-group per (row, key/value head, slice of keys) for decoded tokens, short portions and the all-32-bit mode,
// and a matrix-core form for prompts, whose key tile is one page.  Scores, soft-max and weights are 32-bit in both; the
// matrix-core form hands its float weights to the value product as three bfloat16 parts that add up to all 24 bits.
#include "cai_layered.hpp"
#include "cai_gemv_common.hpp"

#include <algorithm>

namespace cai {

constexpr int SLICE = 64;                  // keys per work-group of the row form: a slice lies in at most two pages

template <typename T> __device__ __forceinline__ float round_to(float v) { return (float)(T)v; }
template <typename T> __device__ __forceinline__ void load8(const T* p, float* v)
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
template <typename T> __device__ __forceinline__ T* kv_page(const KvView& kv, int slot, int key)
{
  return reinterpret_cast<T*>(kv.base) + (int64_t)kv.table[slot * kv.ring + (key / PAGE_TOKENS) % kv.ring] * kv.page_elems;
}

// What all query heads (or key heads) of a row share: the RMS norm's factor under whole_norm, and the queries' growth.
struct RowFactors { float inv_q = 1.0f, inv_k = 1.0f, temp = 1.0f; };
// by a work-group of 256, over the columns of proj; red: LDS for 8 floats
__device__ __forceinline__ RowFactors row_factors(const AttnDims& d, const AttnIn& in, const float* p, int pos, bool with_k, float* red)
{
  RowFactors f;
  if (d.temp_every) f.temp = 1.0f + d.temp * logf((float)((pos + 1) / d.temp_every + 1));
  if (!d.whole_norm) return f;
  const int tid = threadIdx.x, nq = d.heads * d.dim, nk = with_k ? d.kv_heads * d.dim : 0;
  float q = 0.0f, k = 0.0f;
#pragma unroll 8
  for (int c = tid; c < nq; c += 256) { const float v = p[in.oq + c]; q = fmaf(v, v, q); }
#pragma unroll 4
  for (int c = tid; c < nk; c += 256) { const float v = p[in.ok + c]; k = fmaf(v, v, k); }
  q = wave_sum(q); k = wave_sum(k);
  if ((tid & 63) == 63) { red[tid >> 6] = q; red[4 + (tid >> 6)] = k; }
  __syncthreads();
  f.inv_q = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)nq + d.eps);
  if (with_k) f.inv_k = 1.0f / sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)nk + d.eps);
  return f;
}

// weight of a key `far` positions before the query, from the scaled product of the two
__device__ __forceinline__ float sigmoid_weight(const AttnDims& d, int h, float score, int far)
{
  return 1.0f / (1.0f + expf(-(score - d.r1[h] * logf(1.0f + d.r2[h] * (float)far) + d.bias[h])));
}

// A query or key head of `dim` values by one wave, lane holds x[lane + 64 i]: RMS norm (gain null: none) with the factor `inv` or, without
// whole_norm, one of its own, then the rotation at position pos, then `times`.  The angle is reduced in turns with double precision
// before sine and cosine.
__device__ __forceinline__ void head_vector(const float* x, const float* gain, float inv, const float times, const AttnDims& d, int pos, int lane, float* v)
{
  float s = 0.0f;
#pragma unroll
  for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; v[i] = c < d.dim ? x[c] : 0.0f; s = fmaf(v[i], v[i], s); }
  if (gain) {
    s = wave_sum(s);
    if (!d.whole_norm) inv = 1.0f / sqrtf(__builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, s), 63)) / (float)d.dim + d.eps);
#pragma unroll
    for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; if (c < d.dim) v[i] *= inv * gain[c]; }
  }
  const int half = d.rot / 2;
#pragma unroll
  for (int i = 0; i < 4; i++) {
    const int c = lane + 64 * i;
    if (c >= d.rot) continue;
    const bool lo = c < half;
    const int j = lo ? c : c - half, other = lo ? c + half : j;
    float o = x[other];
    if (gain) o *= inv * gain[other];
    const double t = (double)pos * d.turns[j];
    float sn, cs;
    sincospif((float)(2.0 * (t - rint(t))), &sn, &cs);
    v[i] = lo ? v[i] * cs - o * sn : v[i] * cs + o * sn;
  }
#pragma unroll
  for (int i = 0; i < 4; i++) v[i] *= times;
}
__device__ __forceinline__ float out_gate(const AttnIn& in, int64_t row, int c)
{
  return in.og < 0 ? 1.0f : 1.0f / (1.0f + expf(-in.proj[row * in.ldp + in.og + c]));
}

template <typename T>
__global__ __launch_bounds__(256) void attn_prep_kernel(const AttnDims d, const KvView kv, const AttnIn in, const StepRows r, T* qbuf)
{
  const int row = blockIdx.x, lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  __shared__ float red[8];
  const int pos = r.pos[row], slot = r.slot[row], tp = pos % PAGE_TOKENS;
  const float* p = in.proj + row * in.ldp;
  const bool append = in.ok >= 0;
  const RowFactors f = row_factors(d, in, p, pos, append, red);
  T* page = kv_page<T>(kv, slot, pos);
  const int by_head = d.whole_norm ? d.dim : 0;            // gains of one head after the other, or shared
  for (int u = wave; u < d.heads + (append ? d.kv_heads : 0); u += 4) {
    const bool is_q = u < d.heads; const int hh = is_q ? u : u - d.heads;
    const float* gain = is_q ? in.qn : in.kn;
    float v[4];
    head_vector(p + (is_q ? in.oq : in.ok) + hh * d.dim, gain ? gain + hh * by_head : nullptr, is_q ? f.inv_q : f.inv_k, is_q ? f.temp : 1.0f, d, pos, lane, v);
    T* dst = is_q ? qbuf + ((int64_t)row * d.heads + hh) * d.dim_p : page + ((int64_t)hh * PAGE_TOKENS + tp) * d.dim_p;
#pragma unroll
    for (int i = 0; i < 4; i++) { const int c = lane + 64 * i; if (c < d.dim_p) dst[c] = (T)v[i]; }
  }
  if (append) for (int c = threadIdx.x; c < d.kv_heads * d.vdim_p; c += 256) {
    const int hh = c / d.vdim_p, i = c % d.vdim_p;
    page[kv.v_off + ((int64_t)hh * PAGE_TOKENS + tp) * d.vdim_p + i] = (T)(i < d.vdim ? p[in.ov + hh * d.vdim + i] : 0.0f);
  }
}

// ------------------------------------------------------------------------------------------
// Row form.  blockIdx: x slice, y = key/value head x group of HT query heads, z row.  SINGLE: the row is its entry's only one;
// queries, the new key and the new value come from the projections and the new key/value are appended on the way (unless an earlier
// run has filled the pages).
// part (more than one slice): per (row, head, slice) vdim_p weighted sums, the maximum and the normaliser (of a soft-max).
// ------------------------------------------------------------------------------------------
template <typename T, int HT, bool SINGLE>
__global__ __launch_bounds__(256) void attn_rows_kernel(const AttnDims d, const KvView kv, const AttnIn in, const StepRows r, const T* qbuf, T* out, const int64_t ldo, float* part)
{
  __shared__ float sq[HT][256], nk[256], nv[256];
  __shared__ float sc[HT][SLICE];
  __shared__ float red[4][HT][256];
  __shared__ float smax[HT], ssum[HT], rf[8];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int hg = d.heads / d.kv_heads, hblk = (hg + HT - 1) / HT;
  const int row = blockIdx.z, g = blockIdx.y / hblk, h0 = g * hg + blockIdx.y % hblk * HT, nh = min(HT, (g + 1) * hg - h0);
  const int pos = r.pos[row], slot = r.slot[row];
  const int lo = d.first_key(pos), k0 = lo + blockIdx.x * SLICE, nkeys = min(SLICE, pos + 1 - k0);
  const int n_sl = gridDim.x;
  if (nkeys <= 0) {                        // (part is only read up to the slices in use)
    return;
  }
  const bool own_new = SINGLE && in.ok >= 0 && k0 + nkeys == pos + 1;
  // The slice's keys are requested first: sixteen lanes a key, eight elements a lane and turn, four keys a lane group.  A slice lies
  // in at most two pages; a single row's own key is not in its page yet and comes from LDS below (columns past the width meet zeros
  // in the query).
  const int l16 = lane & 15, kb = wave * 4 + (lane >> 4);
  const int pk = (k0 / PAGE_TOKENS + 1) * PAGE_TOKENS;                 // first key of the second page
  const T* pg0 = kv_page<T>(kv, slot, k0), *pg1 = kv_page<T>(kv, slot, k0 + nkeys - 1);
  float kx[4][2][8];
#pragma unroll
  for (int u = 0; u < 4; u++) {
    const int key = k0 + max(0, min(kb + 16 * u, nkeys - 1 - (own_new ? 1 : 0)));
    const T* kp = (key < pk ? pg0 : pg1) + ((int64_t)g * PAGE_TOKENS + key % PAGE_TOKENS) * d.dim_p;
#pragma unroll
    for (int t = 0; t < 2; t++) {
      if (t && d.dim_p <= 128) continue;
      const int c = l16 * 8 + t * 128;
      load8<T>(kp + (c < d.dim_p ? c : 0), kx[u][t]);
    }
  }
  if (SINGLE) {
    const float* p = in.proj + row * in.ldp;
    const RowFactors f = row_factors(d, in, p, pos, own_new, rf);
    for (int u = wave; u < nh + (own_new ? 1 : 0); u += 4) {
      float v[4];
      const bool is_q = u < nh;
      const int hh = is_q ? h0 + u : g;
      const float* gain = is_q ? in.qn : in.kn;
      head_vector(p + (is_q ? in.oq : in.ok) + hh * d.dim, gain && d.whole_norm ? gain + hh * d.dim : gain, is_q ? f.inv_q : f.inv_k, is_q ? f.temp : 1.0f, d, pos, lane, v);
      float* dst = is_q ? sq[u] : nk;
#pragma unroll
      for (int i = 0; i < 4; i++) dst[lane + 64 * i] = is_q ? v[i] : round_to<T>(v[i]);
    }
    if (own_new) for (int c = tid; c < 256; c += 256) nv[c] = c < d.vdim ? round_to<T>(p[in.ov + g * d.vdim + c]) : 0.0f;
  } else {
    for (int i = tid; i < nh * 256; i += 256) {
      const int hh = i >> 8, c = i & 255;
      sq[hh][c] = c < d.dim_p ? (float)qbuf[((int64_t)row * d.heads + h0 + hh) * d.dim_p + c] : 0.0f;
    }
  }
  __syncthreads();
  if (own_new && blockIdx.y % hblk == 0) {
    T* page = kv_page<T>(kv, slot, pos);
    const int tp = pos % PAGE_TOKENS;
    for (int c = tid; c < d.dim_p; c += 256) page[((int64_t)g * PAGE_TOKENS + tp) * d.dim_p + c] = (T)nk[c];
    for (int c = tid; c < d.vdim_p; c += 256) page[kv.v_off + ((int64_t)g * PAGE_TOKENS + tp) * d.vdim_p + c] = (T)nv[c];
  }
  // scores of a lane group's four keys
#pragma unroll
  for (int hh = 0; hh < HT; hh++) {
    if (hh >= nh) break;
    float s[4] = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int t = 0; t < 2; t++) {
      if (t && d.dim_p <= 128) continue;
      float q[8];
      *reinterpret_cast<f32x4*>(q) = *reinterpret_cast<const f32x4*>(&sq[hh][l16 * 8 + t * 128]);
      *reinterpret_cast<f32x4*>(q + 4) = *reinterpret_cast<const f32x4*>(&sq[hh][l16 * 8 + t * 128 + 4]);
#pragma unroll
      for (int u = 0; u < 4; u++) {
        const bool fresh = own_new && kb + 16 * u == nkeys - 1;
#pragma unroll
        for (int i = 0; i < 8; i++) s[u] = fmaf(q[i], fresh ? nk[l16 * 8 + t * 128 + i] : kx[u][t][i], s[u]);
      }
    }
#pragma unroll
    for (int u = 0; u < 4; u++) {
      s[u] += __shfl_xor(s[u], 8); s[u] += __shfl_xor(s[u], 4); s[u] += __shfl_xor(s[u], 2); s[u] += __shfl_xor(s[u], 1);
      if (l16 == 0) sc[hh][kb + 16 * u] = s[u] * d.scale;
    }
  }
  __syncthreads();
  // weights over the slice, a wave per head
  if (d.sigmoid) {
    for (int hh = wave; hh < nh; hh += 4) {
#pragma unroll
      for (int i = 0; i < SLICE / 64; i++) {
        const int k = lane + 64 * i;
        sc[hh][k] = k < nkeys ? sigmoid_weight(d, h0 + hh, sc[hh][k], pos - k0 - k) : 0.0f;
      }
      if (lane == 0) { smax[hh] = 0.0f; ssum[hh] = 1.0f; }
    }
  } else for (int hh = wave; hh < nh; hh += 4) {
    float v[SLICE / 64], m = -INFINITY;
#pragma unroll
    for (int i = 0; i < SLICE / 64; i++) { v[i] = lane + 64 * i < nkeys ? sc[hh][lane + 64 * i] : -INFINITY; m = fmaxf(m, v[i]); }
#pragma unroll
    for (int o = 32; o; o >>= 1) m = fmaxf(m, __shfl_xor(m, o));
    float s = 0.0f;
#pragma unroll
    for (int i = 0; i < SLICE / 64; i++) { v[i] = expf(v[i] - m); s += v[i]; sc[hh][lane + 64 * i] = v[i]; }
#pragma unroll
    for (int o = 32; o; o >>= 1) s += __shfl_xor(s, o);
    if (lane == 0) { smax[hh] = m; ssum[hh] = d.sink && n_sl == 1 ? s + expf(d.sink[h0 + hh] - m) : s; }
  }
  __syncthreads();
  // weighted values: CB lanes along the columns (eight each), the rest of the work-group along the keys
  const int chunks = d.vdim_p / 8;
  int cb_log = 0; while ((1 << cb_log) < chunks) cb_log++;
  const int cbl = 1 << cb_log, cc = tid & (cbl - 1), kg = tid >> cb_log, nkg = 256 >> cb_log;
  float acc[HT][8];
#pragma unroll
  for (int hh = 0; hh < HT; hh++)
#pragma unroll
    for (int i = 0; i < 8; i++) acc[hh][i] = 0.0f;
  if (cc < chunks) {
    for (int kb = kg; kb < nkeys; kb += nkg * 4) {
      float vx[4][8];
#pragma unroll
      for (int u = 0; u < 4; u++) {
        const int key = k0 + min(kb + nkg * u, nkeys - 1);
        if (own_new && key == pos) {
#pragma unroll
          for (int i = 0; i < 8; i++) vx[u][i] = nv[cc * 8 + i];
        } else load8<T>((key < pk ? pg0 : pg1) + kv.v_off + ((int64_t)g * PAGE_TOKENS + key % PAGE_TOKENS) * d.vdim_p + cc * 8, vx[u]);
      }
#pragma unroll
      for (int hh = 0; hh < HT; hh++) {
        if (hh >= nh) break;
#pragma unroll
        for (int u = 0; u < 4; u++) {
          const int kk = kb + nkg * u;
          const float p = kk < nkeys ? sc[hh][kk] : 0.0f;
#pragma unroll
          for (int i = 0; i < 8; i++) acc[hh][i] = fmaf(p, vx[u][i], acc[hh][i]);
        }
      }
    }
  }
#pragma unroll
  for (int hh = 0; hh < HT; hh++) {
    if (hh >= nh) break;
    for (int o = cbl; o < 64; o <<= 1)
#pragma unroll
      for (int i = 0; i < 8; i++) acc[hh][i] += __shfl_xor(acc[hh][i], o);
    if (lane < cbl && cc < chunks) {
      *reinterpret_cast<f32x4*>(&red[wave][hh][cc * 8]) = f32x4{acc[hh][0], acc[hh][1], acc[hh][2], acc[hh][3]};
      *reinterpret_cast<f32x4*>(&red[wave][hh][cc * 8 + 4]) = f32x4{acc[hh][4], acc[hh][5], acc[hh][6], acc[hh][7]};
    }
  }
  __syncthreads();
  for (int i = tid; i < nh * d.vdim_p; i += 256) {
    const int hh = i / d.vdim_p, c = i % d.vdim_p;
    const float s = red[0][hh][c] + red[1][hh][c] + red[2][hh][c] + red[3][hh][c];
    if (n_sl == 1) { if (c < d.vdim) out[row * ldo + (h0 + hh) * d.vdim + c] = (T)(s / ssum[hh] * out_gate(in, row, (h0 + hh) * d.vdim + c)); }
    else part[(((int64_t)row * d.heads + h0 + hh) * n_sl + blockIdx.x) * (d.vdim_p + 2) + c] = s;
  }
  if (n_sl > 1 && tid < nh) {
    float* q = part + (((int64_t)row * d.heads + h0 + tid) * n_sl + blockIdx.x) * (d.vdim_p + 2) + d.vdim_p;
    q[0] = smax[tid]; q[1] = ssum[tid];
  }
}

template <typename T>
__global__ __launch_bounds__(256) void attn_rows_merge_kernel(const AttnDims d, const AttnIn in, const StepRows r, const int n_sl, const float* part, T* out, const int64_t ldo)
{
  __shared__ float sm[4], sl[4], sw[256];
  const int h = blockIdx.x, row = blockIdx.y, pos = r.pos[row], tid = threadIdx.x;
  const int used = (pos - d.first_key(pos) + SLICE) / SLICE, st = d.vdim_p + 2;
  const float* p = part + ((int64_t)row * d.heads + h) * n_sl * st;
  float m = -INFINITY, l = 0.0f;
  if (d.sigmoid) {                         // plain sums
    if (tid < 4) sl[tid] = 0.25f;
  } else {
    for (int s = tid; s < used; s += 256) m = fmaxf(m, p[s * st + d.vdim_p]);
    for (int o = 32; o; o >>= 1) m = fmaxf(m, __shfl_xor(m, o));
    if ((tid & 63) == 0) sm[tid >> 6] = m;
    __syncthreads();
    m = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
    for (int s = tid; s < used; s += 256) l += p[s * st + d.vdim_p + 1] * expf(p[s * st + d.vdim_p] - m);
    for (int o = 32; o; o >>= 1) l += __shfl_xor(l, o);
    if (d.sink && tid == 0) l += expf(d.sink[h] - m);    // (counts once, whatever the number of slices)
    if ((tid & 63) == 0) sl[tid >> 6] = l;
  }
  float acc = 0.0f;
  for (int s0 = 0; s0 < used; s0 += 256) {               // a block of slice weights at a time
    const int ns = min(256, used - s0);
    __syncthreads();
    if (tid < ns) sw[tid] = d.sigmoid ? 1.0f : expf(p[(s0 + tid) * st + d.vdim_p] - m);
    __syncthreads();
    if (tid < d.vdim) {
      for (int s = 0; s < ns; s += 8) {
        float t[8];
#pragma unroll
        for (int u = 0; u < 8; u++) t[u] = p[(s0 + min(s + u, ns - 1)) * st + tid];
#pragma unroll
        for (int u = 0; u < 8; u++) if (s + u < ns) acc = fmaf(t[u], sw[s + u], acc);
      }
    }
  }
  if (tid < d.vdim) out[row * ldo + h * d.vdim + tid] = (T)(acc / (sl[0] + sl[1] + sl[2] + sl[3]) * out_gate(in, row, h * d.vdim + tid));
}

// ------------------------------------------------------------------------------------------
// Prompt form: 64 query rows of one entry and one head per work-group, a wave per 16 rows; a key tile is a page.
// S^T = K Q^T puts a query in a lane column, so its soft-max state is per lane; the score registers are the B operand of
// O^T = V^T P^T as they are: key slot (lane group g, j) of a 32-key step is key 4 g + j of its first 16 keys for j < 4 and
// 4 g + j - 4 of its second 16 otherwise, and V^T is read from LDS in that order.
// ------------------------------------------------------------------------------------------
template <int KQ, int VQ, bool SIG, bool FLAT>   // key width in 32s, value width in 16s; sigmoid weights; keys and values in rows (FlatKv)
__global__ __launch_bounds__(256) void attn_prompt_paged_kernel(const AttnDims d, const KvView kv, const FlatKv flat, const AttnIn in, const bf16_t* qbuf, const StepRows r, const int32_t* tiles, bf16_t* out, const int64_t ldo)
{
  constexpr int KST = KQ * 32 + 8, VST = PAGE_TOKENS + 4;
  __shared__ __align__(16) uint16_t sk[PAGE_TOKENS * KST];
  __shared__ __align__(16) uint16_t sv[VQ * 16 * VST];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), fr = lane & 15, fg = lane >> 4;
  // with key/value heads in whole eights, everything that reads one of them runs on one XCD (consecutive work-groups go to
  // different ones), heads of a group and neighbouring tiles next to each other
  const int hg = d.heads / d.kv_heads;
  int tile = blockIdx.x, h = blockIdx.y;
  if (d.kv_heads % 8 == 0) {
    const int id = blockIdx.x + gridDim.x * blockIdx.y, j = id >> 3;
    h = ((id & 7) + 8 * (j / (hg * (int)gridDim.x))) * hg + j % hg;
    tile = j / hg % gridDim.x;
  }
  const int32_t* en = r.ent + 4 * tiles[2 * tile];
  const int slot = en[0], row0 = en[1], n = en[2], pos0 = en[3], t0 = tiles[2 * tile + 1];
  const int g = h / hg;
  const int qi = t0 + wave * 16 + fr, qr = min(qi, n - 1), qpos = pos0 + qr, qlo = d.first_key(qpos);
  u32x4 fq[KQ];
#pragma unroll
  for (int k = 0; k < KQ; k++) {
    const int c = k * 32 + fg * 8;
    fq[k] = u32x4{0, 0, 0, 0};
    if (c < d.dim_p) fq[k] = *reinterpret_cast<const u32x4*>(qbuf + ((int64_t)(row0 + qr) * d.heads + h) * d.dim_p + c);
  }
  f32x4 o[VQ];
#pragma unroll
  for (int v = 0; v < VQ; v++) o[v] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  float m = -INFINITY, l = 0.0f;
  const int first = d.first_key(pos0 + t0) / PAGE_TOKENS, last = (pos0 + min(t0 + ATTN_TILE, n) - 1) / PAGE_TOKENS;
  const int wmin = pos0 + min(t0 + wave * 16, n - 1), whi = pos0 + min(t0 + wave * 16 + 15, n - 1);   // the wave's first and last row
  // sigmoid weights: 1 / (1 + 2^(cs score + r1 log2(1 + r2 far) - bias log2 e))
  const float cs = SIG ? -d.scale * 1.44269504088896340736f : 0.0f, dr1 = SIG ? d.r1[h] : 0.0f, dr2 = SIG ? d.r2[h] : 0.0f, db = SIG ? -1.44269504088896340736f * d.bias[h] : 0.0f;
  const int wlo = d.first_key(wmin), wall = d.first_key(whi);         // first key any of its rows sees, first key all of them see
  const float scale2 = d.scale * 1.44269504088896340736f;             // scores in base-2 logarithms
  constexpr int KC = PAGE_TOKENS * KQ * 4 / 256, VC = PAGE_TOKENS / 2 * VQ * 2 / 256;   // 16-byte key chunks / value chunk pairs per thread
  u32x4 rk[KC], rv[VC][2];
  // value chunks: eight lanes along pairs of keys, then along the columns, so that the transposing LDS writes spread over the banks
  auto vtok = [](int e) { return ((e & 7) + (e / (VQ * 2 * 8)) * 8) * 2; };
  auto vcol = [](int e) { return (e >> 3) % (VQ * 2) * 8; };
  int page_no = kv.table[slot * kv.ring + first % kv.ring];
  const bf16_t* flat_rows = FLAT ? reinterpret_cast<const bf16_t*>(flat.base) + (int64_t)flat.row0[tiles[2 * tile]] * flat.ld + (int64_t)g * flat.head : nullptr;
  auto fetch = [&](int pg) {
    const bf16_t* page = reinterpret_cast<const bf16_t*>(kv.base) + (int64_t)page_no * kv.page_elems;
    page_no = kv.table[slot * kv.ring + min(pg + 1, last) % kv.ring];      // (the next page's number, a page ahead)
    if constexpr (FLAT) {
      const bf16_t* rows = flat_rows + (int64_t)pg * PAGE_TOKENS * flat.ld;
#pragma unroll
      for (int i = 0; i < KC; i++) {
        const int e = tid + 256 * i, t = e / (KQ * 4), c = e % (KQ * 4) * 8;
        rk[i] = *reinterpret_cast<const u32x4*>(c < flat.split || c >= d.dim_p ? rows + (unsigned)(t * (int)flat.ld + (c < flat.split ? c : 0)) : page + (unsigned)(t * flat.page_row + flat.shared + c - flat.split));
      }
#pragma unroll
      for (int i = 0; i < VC; i++) {
        const int t = vtok(tid + 256 * i), c = vcol(tid + 256 * i);
        const bf16_t* vp = rows + (unsigned)(t * (int)flat.ld + flat.v_off + (c < d.vdim_p ? c : 0));
        rv[i][0] = *reinterpret_cast<const u32x4*>(vp); rv[i][1] = *reinterpret_cast<const u32x4*>(vp + flat.ld);
      }
      return;
    }
#pragma unroll
    for (int i = 0; i < KC; i++) {
      const int e = tid + 256 * i, t = e / (KQ * 4), c = e % (KQ * 4) * 8;
      rk[i] = *reinterpret_cast<const u32x4*>(page + (unsigned)((g * PAGE_TOKENS + t) * d.dim_p + (c < d.dim_p ? c : 0)));
    }
#pragma unroll
    for (int i = 0; i < VC; i++) {
      const int t = vtok(tid + 256 * i), c = vcol(tid + 256 * i);
      const bf16_t* vp = page + kv.v_off + (unsigned)((g * PAGE_TOKENS + t) * d.vdim_p + (c < d.vdim_p ? c : 0));
      rv[i][0] = *reinterpret_cast<const u32x4*>(vp); rv[i][1] = *reinterpret_cast<const u32x4*>(vp + d.vdim_p);
    }
  };
  const int end = pos0 + n;                // keys at and past it are not written yet: their page rows may hold anything
  fetch(first);
  for (int pg = first; pg <= last; pg++) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KC; i++) {
      const int e = tid + 256 * i, t = e / (KQ * 4), c = e % (KQ * 4) * 8;
      *reinterpret_cast<u32x4*>(sk + t * KST + c) = c < d.dim_p ? rk[i] : u32x4{0, 0, 0, 0};
    }
#pragma unroll
    for (int i = 0; i < VC; i++) {
      const int t = vtok(tid + 256 * i), c = vcol(tid + 256 * i);
      const bool k0 = c < d.vdim_p && pg * PAGE_TOKENS + t < end, k1 = c < d.vdim_p && pg * PAGE_TOKENS + t + 1 < end;
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const uint32_t a = k0 ? rv[i][0][j] : 0, b = k1 ? rv[i][1][j] : 0;
        *reinterpret_cast<uint32_t*>(sv + (c + 2 * j) * VST + t) = (a & 0xffffu) | (b << 16);
        *reinterpret_cast<uint32_t*>(sv + (c + 2 * j + 1) * VST + t) = (a >> 16) | (b & 0xffff0000u);
      }
    }
    __syncthreads();
    if (pg < last) fetch(pg + 1);
    if (pg * PAGE_TOKENS > whi || pg * PAGE_TOKENS + PAGE_TOKENS - 1 < wlo) continue;    // (the whole wave: its rows see nothing of this page)
    f32x4 s[4];
#pragma unroll
    for (int t = 0; t < 4; t++) {
      s[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int k = 0; k < KQ; k++) {
        const u32x4 a = *reinterpret_cast<const u32x4*>(sk + (t * 16 + fr) * KST + k * 32 + fg * 8);
        s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, fq[k]), s[t], 0, 0, 0);
      }
    }
    float mt = -INFINITY, mr = 0.0f;
    if constexpr (SIG) {
      const bool whole = pg * PAGE_TOKENS + PAGE_TOKENS - 1 <= wmin && pg * PAGE_TOKENS >= wall;
#pragma unroll
      for (int t = 0; t < 4; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          const int key = pg * PAGE_TOKENS + t * 16 + fg * 4 + i;
          const float far = (float)(qpos - key);
          float z = fmaf(cs, s[t][i], fmaf(dr1, __builtin_amdgcn_logf(fmaf(dr2, whole ? far : fmaxf(far, 0.0f), 1.0f)), db));
          if (!whole && (key > qpos || key < qlo)) z = INFINITY;
          s[t][i] = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z));
        }
    } else if (pg * PAGE_TOKENS + PAGE_TOKENS - 1 <= wmin && pg * PAGE_TOKENS >= wall) {   // every row of the wave sees the whole page
#pragma unroll
      for (int t = 0; t < 4; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) { s[t][i] *= scale2; mt = fmaxf(mt, s[t][i]); }
    } else {
#pragma unroll
      for (int t = 0; t < 4; t++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          const int key = pg * PAGE_TOKENS + t * 16 + fg * 4 + i;
          s[t][i] = key <= qpos && key >= qlo ? s[t][i] * scale2 : -INFINITY;
          mt = fmaxf(mt, s[t][i]);
        }
    }
    if constexpr (!SIG) {
      mt = fmaxf(mt, __shfl_xor(mt, 16)); mt = fmaxf(mt, __shfl_xor(mt, 32));
      const float mn = fmaxf(m, mt);
      mr = mn == -INFINITY ? 0.0f : mn;
      const float al = __builtin_amdgcn_exp2f(m - mr);
      m = mn; l *= al;
#pragma unroll
      for (int v = 0; v < VQ; v++) o[v] *= al;
    }
    // weights in three bfloat16 parts, p = p0 + p1 + p2 exactly (upper halves of p and of what is left)
    uint32_t w[3][16];
#pragma unroll
    for (int t = 0; t < 4; t++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const float p = SIG ? s[t][i] : __builtin_amdgcn_exp2f(s[t][i] - mr);
        if constexpr (!SIG) l += p;
        const uint32_t b0 = __builtin_bit_cast(uint32_t, p);
        const float r1 = p - __builtin_bit_cast(float, b0 & 0xffff0000u);
        const uint32_t b1 = __builtin_bit_cast(uint32_t, r1);
        w[0][t * 4 + i] = b0; w[1][t * 4 + i] = b1;
        w[2][t * 4 + i] = __builtin_bit_cast(uint32_t, r1 - __builtin_bit_cast(float, b1 & 0xffff0000u));
      }
#pragma unroll
    for (int hp = 0; hp < 2; hp++) {
      u32x4 fp[3];
#pragma unroll
      for (int q = 0; q < 3; q++)
#pragma unroll
        for (int j = 0; j < 4; j++) fp[q][j] = __builtin_amdgcn_perm(w[q][hp * 8 + 2 * j + 1], w[q][hp * 8 + 2 * j], 0x07060302);   // upper halves of two words
#pragma unroll
      for (int v = 0; v < VQ; v++) {
        const uint16_t* vr = sv + (v * 16 + fr) * VST + hp * 32 + fg * 4;
        const uint2 lo2 = *reinterpret_cast<const uint2*>(vr), hi2 = *reinterpret_cast<const uint2*>(vr + 16);
        const u32x4 a = {lo2.x, lo2.y, hi2.x, hi2.y};
#pragma unroll
        for (int q = 0; q < 3; q++) o[v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, fp[q]), o[v], 0, 0, 0);
      }
    }
  }
  l += __shfl_xor(l, 16); l += __shfl_xor(l, 32);
  if (!SIG && d.sink) l += __builtin_amdgcn_exp2f(d.sink[h] * 1.44269504088896340736f - m);
  if (qi < n) {
    const float inv = SIG ? 1.0f : 1.0f / l;
#pragma unroll
    for (int v = 0; v < VQ; v++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int c = v * 16 + fg * 4 + i;
        if (c < d.vdim) out[(int64_t)(row0 + qi) * ldo + h * d.vdim + c] = (bf16_t)(o[v][i] * inv * out_gate(in, row0 + qi, h * d.vdim + c));
      }
  }
}

int attn_paged_prep(const AttnDims& d, const KvView& kv, int act_t, const AttnIn& in, const StepRows& r, void* qbuf)
{
  if (act_t == ACT_T_BF16) hipLaunchKernelGGL(attn_prep_kernel<bf16_t>, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, kv, in, r, (bf16_t*)qbuf);
  else hipLaunchKernelGGL(attn_prep_kernel<float>, dim3(r.n_rows), dim3(256), 0, ctx().stream, d, kv, in, r, (float*)qbuf);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

static int n_slices(const AttnDims& d, int reach) { return (std::min(d.span, reach) + SLICE - 1) / SLICE; }
constexpr size_t PART_FLOATS = 64 << 20;   // partial results of more rows than fit this are made in turns
static size_t part_row(const AttnDims& d, int ns) { return (size_t)d.heads * ns * (d.vdim_p + 2); }
size_t attn_paged_part_floats(const AttnDims& d, int n_rows)
{
  const int ns = n_slices(d, d.span);
  return ns > 1 ? std::max(part_row(d, ns), std::min(PART_FLOATS, (size_t)n_rows * part_row(d, ns))) : 0;
}

template <typename T, int HT>
static void run_rows(const AttnDims& d, const KvView& kv, const AttnIn& in, const StepRows& r, const T* qbuf, T* out, int64_t ldo, float* part, bool single)
{
  const int hg = d.heads / d.kv_heads, ns = n_slices(d, r.reach);
  const dim3 grid(ns, d.kv_heads * ((hg + HT - 1) / HT), r.n_rows);
  if (single) hipLaunchKernelGGL((attn_rows_kernel<T, HT, true>), grid, dim3(256), 0, ctx().stream, d, kv, in, r, qbuf, out, ldo, part);
  else hipLaunchKernelGGL((attn_rows_kernel<T, HT, false>), grid, dim3(256), 0, ctx().stream, d, kv, in, r, qbuf, out, ldo, part);
  if (ns > 1) hipLaunchKernelGGL(attn_rows_merge_kernel<T>, dim3(d.heads, r.n_rows), dim3(256), 0, ctx().stream, d, in, r, ns, part, out, ldo);
}
template <typename T>
static void run_rows_t(const AttnDims& d, const KvView& kv, const AttnIn& in, const StepRows& r, const void* qbuf, void* out, int64_t ldo, float* part, bool single)
{
  const int hg = d.heads / d.kv_heads;
  if (hg == 1) run_rows<T, 1>(d, kv, in, r, (const T*)qbuf, (T*)out, ldo, part, single);
  else if (hg == 2) run_rows<T, 2>(d, kv, in, r, (const T*)qbuf, (T*)out, ldo, part, single);
  else run_rows<T, 4>(d, kv, in, r, (const T*)qbuf, (T*)out, ldo, part, single);
}
int attn_paged_rows(const AttnDims& d, const KvView& kv, int act_t, const void* qbuf, const StepRows& r, void* out, int64_t ldo, float* part, size_t part_floats, bool single, const AttnIn& in)
{
  const int ns = n_slices(d, r.reach);
  size_t turn = 32768;                     // rows of one launch
  if (ns > 1) turn = std::min(turn, part_floats / part_row(d, ns));
  CAI_REQUIRE(turn >= 1, "attention: partial results of %d slices do not fit %zu floats", ns, part_floats);
  const size_t es = act_t == ACT_T_BF16 ? 2 : 4;
  for (int r0 = 0; r0 < r.n_rows; r0 += (int)turn) {
    StepRows q = r; AttnIn a = in;
    q.pos += r0; q.slot += r0; q.n_rows = std::min((int)turn, r.n_rows - r0);
    a.proj += r0 * in.ldp;
    const char* qb = (const char*)qbuf + (size_t)r0 * d.heads * d.dim_p * es;
    char* o = (char*)out + (size_t)r0 * ldo * es;
    if (act_t == ACT_T_BF16) run_rows_t<bf16_t>(d, kv, a, q, qb, o, ldo, part, single);
    else run_rows_t<float>(d, kv, a, q, qb, o, ldo, part, single);
  }
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

bool attn_paged_prompt_ok(const AttnDims& d, int act_t) { return act_t == ACT_T_BF16 && d.dim <= 256 && d.vdim <= 256; }

int attn_paged_prompt(const AttnDims& d, const KvView& kv, const AttnIn& in, const void* qbuf, const StepRows& r, const int32_t* tiles, int n_tiles, void* out, int64_t ldo)
{
  const dim3 grid(n_tiles, d.heads), blk(256);
#define PROMPT_S(K, V, S, F) hipLaunchKernelGGL((attn_prompt_paged_kernel<K, V, S, F>), grid, blk, 0, ctx().stream, d, kv, f, in, (const bf16_t*)qbuf, r, tiles, (bf16_t*)out, ldo)
#define PROMPT_V(K, P) do { if (d.vdim <= 64) P(K, 4); else if (d.vdim <= 128) P(K, 8); else P(K, 16); } while (0)
#define PROMPT_K(P) do { if (d.dim <= 64) PROMPT_V(2, P); else if (d.dim <= 128) PROMPT_V(4, P); else if (d.dim <= 192) PROMPT_V(6, P); else PROMPT_V(8, P); } while (0)
#define PAGED(K, V) do { if (d.sigmoid) PROMPT_S(K, V, true, false); else PROMPT_S(K, V, false, false); } while (0)
  const FlatKv f;
  PROMPT_K(PAGED);
#undef PAGED
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int attn_flat_prompt(const AttnDims& d, const KvView& kv, const FlatKv& f, const AttnIn& in, const void* qbuf, const StepRows& r, const int32_t* tiles, int n_tiles, void* out, int64_t ldo)
{
  CAI_REQUIRE(!d.sigmoid && f.base && f.row0 && f.split % 8 == 0 && f.shared % 8 == 0 && f.ld % 8 == 0 && f.ld < (1 << 24), "attention over rows: %d shared columns from %d, rows of %lld", f.shared, f.split, (long long)f.ld);
  const dim3 grid(n_tiles, d.heads), blk(256);
#define FLAT(K, V) PROMPT_S(K, V, false, true)
  PROMPT_K(FLAT);
#undef FLAT
#undef PROMPT_K
#undef PROMPT_V
#undef PROMPT_S
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

}  // namespace cai
