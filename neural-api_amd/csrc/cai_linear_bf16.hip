// Linear layers over bfloat16 weights: a streaming matrix-vector kernel for up to eight activation rows (decode) and a
// matrix-core kernel for more (prompts and mixed batches).
//
// Weights are row-major [out][padded in], the padding zero.  Activations are bfloat16 (matrix cores multiply bfloat16 with
// 32-bit sums) or float; with float activations the weights are widened exactly and every product and sum is 32-bit (the
// 16x16x4 float form of the matrix cores).  What follows the product runs in its epilogue on the 32-bit sums: bias and
// activation, act(gate) * up of a gated pair, or the residual update with the Dynamic Tanh before and after it - that norm
// has no statistics, so a sublayer needs no launch besides its products and its mixer - or a result's scaled and gated joining.  The
// streaming kernel takes float rows (the stream's) through an RMS norm itself, and runs two products in one launch.  The matrix-core kernel also runs over a
// bank of equal matrices with a list of activation rows for each (mixtures of experts).
#include "cai_lin_epilogue.hpp"

#include <algorithm>

namespace cai {

// ------------------------------------------------------------------------------------------
// Decode: NB activation rows.  A wave owns R weight rows (of a gated matrix R / 2 outputs) or, with ksplit > 1, every ksplit-th
// 512-wide turn of them; the activations are staged in LDS as float in panels, the weights stream past once.
// GV_RMS: the activations are the float stream, RMS-normed on the way (the gain while they are staged, the root at the end), and the
// work-groups from q.blocks on do the same for a second matrix with a gain of its own.
// GV_PAIR: two products over the same outputs, both joined to the stream.
// ------------------------------------------------------------------------------------------
constexpr int GV_WAVES = 8;
constexpr int GV_LDS = 16384;              // most floats of staged activations (a launch asks for what its width needs)
enum { GV_PLAIN = 0, GV_RMS = 1, GV_PAIR = 2 };
struct GvSecond {                          // the second matrix of GV_RMS and GV_PAIR, and what the norm needs
  const uint16_t* W = nullptr; const void* x = nullptr; int n_rows = 0, ldw = 0; int64_t ldx = 0; LinEpi e;
  int blocks = 0, width = 0; float eps = 0.0f; const float *gain = nullptr, *gain2 = nullptr;
  void *normed = nullptr, *normed2 = nullptr; int64_t ldn = 0;   // the normed rows themselves (null: not)
};

template <typename AT, int NB, int R, int KIND>
__global__ __launch_bounds__(64 * GV_WAVES) void gemv_bf16(const uint16_t* __restrict__ W, const void* __restrict__ xv, int n_rows, int ldw, int64_t ldx, int ksplit, LinEpi e, GvSecond q)
{
  // one row: as much as its width needs (more work-groups fit a CU); several rows: a fixed array, its layout known at compile time
  extern __shared__ float xs_dyn[];
  __shared__ float xs_fix[NB == 1 ? 1 : GV_LDS];
  float* const xs = NB == 1 ? xs_dyn : xs_fix;
  __shared__ float part[GV_WAVES][R * NB];
  __shared__ float sq[GV_WAVES][NB];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int ks = wave % ksplit;
  int block = blockIdx.x, n_blocks = q.blocks;             // (of this matrix)
  const float* gain = q.gain;
  if constexpr (KIND == GV_RMS) {
    if (block >= q.blocks) { block -= q.blocks; n_blocks = gridDim.x - q.blocks; W = q.W; n_rows = q.n_rows; e = q.e; gain = q.gain2; q.normed = q.normed2; }
  }
  const int grp = block * (GV_WAVES / ksplit) + wave / ksplit;
  constexpr int PANEL = GV_LDS / NB / 512 * 512;
  const bool glu = KIND == GV_PLAIN && e.mode == EPI_GLU;
  float ss[NB];                            // sums of squares of the rows
#pragma unroll
  for (int b = 0; b < NB; b++) ss[b] = 0.0f;

  // lane i * NB + b ends with the sum of row i, activation b (of the first wave of a split row)
  auto product = [&](const uint16_t* __restrict__ M, const void* __restrict__ xw, const int ld, const int64_t lx) -> float {
    const AT* x = reinterpret_cast<const AT*>(xw);
    const uint16_t* row[R];
#pragma unroll
    for (int i = 0; i < R; i++) {
      int r = glu ? glu_row(grp * (R / 2) + i % (R / 2 > 0 ? R / 2 : 1), i / (R / 2 > 0 ? R / 2 : 1)) : grp * R + i;
      row[i] = M + (int64_t)min(r, n_rows - 1) * ld;
    }
    float acc[R][NB];
#pragma unroll
    for (int i = 0; i < R; i++)
#pragma unroll
      for (int b = 0; b < NB; b++) acc[i][b] = 0.0f;
    for (int p0 = 0; p0 < ld; p0 += PANEL) {
      const int pk = min(PANEL, ld - p0), pk512 = (pk + 511) / 512 * 512;
      // eight weights a turn ahead of the staging: the first requests are out while the activations arrive
      u32x4 w0[R];
      const int k_first = ks * 512 + lane * 8;
#pragma unroll
      for (int i = 0; i < R; i++) w0[i] = *reinterpret_cast<const u32x4*>(row[i] + p0 + (k_first < pk ? k_first : 0));
      if (p0) __syncthreads();
#pragma unroll
      for (int b = 0; b < NB; b++)
        for (int k = threadIdx.x * 8; k < pk512; k += 64 * GV_WAVES * 8) {
          float v[8];
          if constexpr (KIND == GV_RMS) {
            const float* xf = reinterpret_cast<const float*>(xw) + b * lx;
            const int c = p0 + k;
            if (c + 8 <= q.width && (lx & 3) == 0) {
              const f32x4 a = *reinterpret_cast<const f32x4*>(xf + c), d = *reinterpret_cast<const f32x4*>(xf + c + 4);
              const f32x4 ga = *reinterpret_cast<const f32x4*>(gain + c), gd = *reinterpret_cast<const f32x4*>(gain + c + 4);
#pragma unroll
              for (int j = 0; j < 4; j++) { ss[b] = fmaf(a[j], a[j], ss[b]); ss[b] = fmaf(d[j], d[j], ss[b]); v[j] = a[j] * ga[j]; v[4 + j] = d[j] * gd[j]; }
            } else {
#pragma unroll
              for (int j = 0; j < 8; j++) { const float a = c + j < q.width ? xf[c + j] : 0.0f; ss[b] = fmaf(a, a, ss[b]); v[j] = c + j < q.width ? a * gain[c + j] : 0.0f; }
            }
          } else if (k < pk) {
            if constexpr (sizeof(AT) == 2) {
              const u32x4 u = *reinterpret_cast<const u32x4*>(x + b * lx + p0 + k);
#pragma unroll
              for (int j = 0; j < 4; j++) { v[2 * j] = bf16_lo(u[j]); v[2 * j + 1] = bf16_hi(u[j]); }
            } else {
              const f32x4 a = *reinterpret_cast<const f32x4*>(x + b * lx + p0 + k), c = *reinterpret_cast<const f32x4*>(x + b * lx + p0 + k + 4);
#pragma unroll
              for (int j = 0; j < 4; j++) { v[j] = a[j]; v[4 + j] = c[j]; }
            }
          } else {
#pragma unroll
            for (int j = 0; j < 8; j++) v[j] = 0.0f;
          }
          // a turn of 512 values is kept as two halves of 256 (four values a lane each), so that a wave's 16-byte reads are contiguous
          float* o = xs + b * PANEL + (k >> 9) * 512 + ((k >> 3) & 63) * 4;
          *reinterpret_cast<f32x4*>(o) = f32x4{v[0], v[1], v[2], v[3]};
          *reinterpret_cast<f32x4*>(o + 256) = f32x4{v[4], v[5], v[6], v[7]};
        }
      if constexpr (KIND == GV_RMS) {
        if (p0 + PANEL >= ld)
#pragma unroll
          for (int b = 0; b < NB; b++) { const float t = wave_sum(ss[b]); if (lane == 63) sq[wave][b] = t; }
      }
      __syncthreads();
      for (int k0 = ks * 512; k0 < pk512; k0 += ksplit * 512) {
        u32x4 w1[R];
        const int kn = k0 + ksplit * 512 + lane * 8;
#pragma unroll
        for (int i = 0; i < R; i++) w1[i] = *reinterpret_cast<const u32x4*>(row[i] + p0 + (kn < pk ? kn : 0));
#pragma unroll
        for (int b = 0; b < NB; b++) {
          const f32x4 xa = *reinterpret_cast<const f32x4*>(xs + b * PANEL + k0 + lane * 4);
          const f32x4 xb = *reinterpret_cast<const f32x4*>(xs + b * PANEL + k0 + 256 + lane * 4);
#pragma unroll
          for (int i = 0; i < R; i++) {
            float s = acc[i][b];
            s = fmaf(bf16_lo(w0[i][0]), xa[0], s); s = fmaf(bf16_hi(w0[i][0]), xa[1], s);
            s = fmaf(bf16_lo(w0[i][1]), xa[2], s); s = fmaf(bf16_hi(w0[i][1]), xa[3], s);
            s = fmaf(bf16_lo(w0[i][2]), xb[0], s); s = fmaf(bf16_hi(w0[i][2]), xb[1], s);
            s = fmaf(bf16_lo(w0[i][3]), xb[2], s); s = fmaf(bf16_hi(w0[i][3]), xb[3], s);
            acc[i][b] = s;
          }
        }
#pragma unroll
        for (int i = 0; i < R; i++) w0[i] = w1[i];
      }
    }
    float mine = 0.0f;
#pragma unroll
    for (int i = 0; i < R; i++)
#pragma unroll
      for (int b = 0; b < NB; b++) {
        const float t = wave_sum(acc[i][b]);
        const float s = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, t), 63));
        if (lane == i * NB + b) mine = s;
      }
    if (ksplit > 1) {
      if (lane < R * NB) part[wave][lane] = mine;
      __syncthreads();
      if (ks == 0 && lane < R * NB) for (int j = 1; j < ksplit; j++) mine += part[wave + j][lane];
    }
    return mine;
  };

  float mine = product(W, xv, ldw, ldx);
  const int i = lane / NB, b = lane % NB;
  if constexpr (KIND == GV_PAIR) {
    __syncthreads();
    const float second = product(q.W, q.x, q.ldw, q.ldx);
    if (ks == 0 && i < R && grp * R + i < n_rows) join_two(e, mine, q.e, second, grp * R + i, b);
    return;
  }
  if constexpr (KIND == GV_RMS) {
    auto root = [&](int r) {
      float t = 0.0f;
#pragma unroll
      for (int w = 0; w < GV_WAVES; w++) t += sq[w][r];
      return 1.0f / sqrtf(t / (float)q.width + q.eps);
    };
    mine *= root(b);
    for (int r = block; q.normed && r < NB; r += n_blocks) {   // the first work-groups leave a normed row each
      const float inv = root(r);
      const float* xf = reinterpret_cast<const float*>(xv) + r * ldx;
#pragma unroll 4
      for (int k = threadIdx.x; k < q.ldn; k += 64 * GV_WAVES) put_act<AT>(q.normed, r * q.ldn + k, k < q.width ? xf[k] * inv * gain[k] : 0.0f);
    }
  }
  if (ks != 0) return;
  if (glu) {
    const float up = __shfl(mine, lane + R / 2 * NB);
    const int j = grp * (R / 2) + i;
    if (i < R / 2 && glu_row(j, 0) < n_rows) put_act<AT>(e.h, b * e.ldh + j, glu_pair(e.glu, e.limit, mine, up));
  } else if (i < R && grp * R + i < n_rows) {
    if constexpr (KIND == GV_RMS) { if (e.mode == EPI_SPLIT) epi_as<AT, EPI_SPLIT>(e, grp * R + i, b, mine); else epi_as<AT, EPI_STORE>(e, grp * R + i, b, mine); }
    else epi_one<AT>(e, grp * R + i, b, mine);
  }
}

// ------------------------------------------------------------------------------------------
// Prompts: C^T tile = W tile x activations^T on the matrix cores; a lane ends with four consecutive outputs of one token.
// Both operand tiles are 128 bytes deep per row (64 bfloat16 or 32 floats), double buffered in LDS; the 16-byte chunks of a row
// are stored at chunk ^ (row & 7), which makes the fragment reads conflict-free.
// ------------------------------------------------------------------------------------------
template <typename AT, int BM, int BN, int WM, int WN, bool BANK, int MODE>   // MODE: e.mode (one epilogue a kernel: with all of them the accumulators would leave their registers)
__global__ __launch_bounds__(64 * WM * WN) void gemm_bf16(const uint16_t* __restrict__ W, const AT* __restrict__ X, int n_rows, int ldw, int64_t ldx, int n_tok, int tiles_m, int n_tiles, LinEpi e, BankList l)
{
  constexpr int NT = 64 * WM * WN;
  constexpr int BK = 128 / (int)sizeof(AT);          // elements per row of a tile
  constexpr int TM = BM / WM / 16, TN = BN / WN / 16;
  constexpr int CA = BM * 8 / NT, CW = BN * 8 / NT;  // 16-byte chunks per thread
  static_assert(CA >= 1 && CW >= 1 && BM * 8 % NT == 0 && BN * 8 % NT == 0 && TN % 2 == 0, "tile shape");
  __shared__ u32x4 sx[2][BM * 8], sw[2][BN * 8];
  // consecutive work-groups go to different XCDs: give each XCD a contiguous run of tiles, token tiles fastest, so that the
  // work-groups of an XCD share weight rows in its L2
  int tile;
  {
    const int xcd = blockIdx.x & 7, per = n_tiles >> 3, rem = n_tiles & 7;
    tile = xcd * per + min(xcd, rem) + (blockIdx.x >> 3);
  }
  int m0 = tile % tiles_m * BM;
  const int n0 = tile / tiles_m * BN;
  if constexpr (BANK) {                    // n_rows: of one matrix; the token tile is a run of places of the order
    const int tm = tile % tiles_m;
    if (tm >= *l.n_tiles) return;
    const int32_t* tl = l.tiles + 3 * tm;
    W += (int64_t)tl[0] * n_rows * ldw;
    m0 = tl[1]; n_tok = m0 + tl[2];
  }
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wm = wave / WN * (BM / WM), wn = wave % WN * (BN / WN);
  const AT* xp[CA]; const uint16_t* wp[CW];
#pragma unroll
  for (int i = 0; i < CA; i++) {
    const int c = tid + i * NT;
    int t = min(m0 + (c >> 3), n_tok - 1);
    if constexpr (BANK) { if (l.div) t = l.order[t] / l.div; }
    xp[i] = X + (int64_t)t * ldx + (c & 7) * (16 / sizeof(AT));
  }
#pragma unroll
  for (int i = 0; i < CW; i++) { const int c = tid + i * NT; wp[i] = W + (int64_t)min(n0 + (c >> 3), n_rows - 1) * ldw + (c & 7) * (16 / sizeof(AT)); }
  u32x4 rx[CA], rw[CW];
  auto fetch = [&](int k) {
#pragma unroll
    for (int i = 0; i < CA; i++) rx[i] = *reinterpret_cast<const u32x4*>(xp[i] + k);
#pragma unroll
    for (int i = 0; i < CW; i++) {
      if constexpr (sizeof(AT) == 2) rw[i] = *reinterpret_cast<const u32x4*>(wp[i] + k);
      else {
        const uint2 u = *reinterpret_cast<const uint2*>(wp[i] + k);
        rw[i] = u32x4{u.x << 16, u.x & 0xffff0000u, u.y << 16, u.y & 0xffff0000u};
      }
    }
  };
  auto stash = [&](int s) {
#pragma unroll
    for (int i = 0; i < CA; i++) { const int c = tid + i * NT, r = c >> 3; sx[s][r * 8 + ((c & 7) ^ (r & 7))] = rx[i]; }
#pragma unroll
    for (int i = 0; i < CW; i++) { const int c = tid + i * NT, r = c >> 3; sw[s][r * 8 + ((c & 7) ^ (r & 7))] = rw[i]; }
  };
  f32x4 acc[TN][TM];
#pragma unroll
  for (int j = 0; j < TN; j++)
#pragma unroll
    for (int i = 0; i < TM; i++) acc[j][i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  const int fr = lane & 15, fc = lane >> 4;
  fetch(0); stash(0);
  __syncthreads();
  const int nk = ldw / BK;
  for (int kt = 0; kt < nk; kt++) {
    const int s = kt & 1;
    if (kt + 1 < nk) fetch((kt + 1) * BK);
#pragma unroll
    for (int kk = 0; kk < 2; kk++) {
      u32x4 fx[TM], fw[TN];
#pragma unroll
      for (int i = 0; i < TM; i++) { const int r = wm + i * 16 + fr; fx[i] = sx[s][r * 8 + ((kk * 4 + fc) ^ (r & 7))]; }
#pragma unroll
      for (int j = 0; j < TN; j++) { const int r = wn + j * 16 + fr; fw[j] = sw[s][r * 8 + ((kk * 4 + fc) ^ (r & 7))]; }
#pragma unroll
      for (int j = 0; j < TN; j++)
#pragma unroll
        for (int i = 0; i < TM; i++) {
          if constexpr (sizeof(AT) == 2) {
            acc[j][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, fw[j]), __builtin_bit_cast(bf16x8, fx[i]), acc[j][i], 0, 0, 0);
          } else {
            // the k index a lane group contributes at step q is 4 * group + q of the 16-wide block, for both operands alike
            const f32x4 a = __builtin_bit_cast(f32x4, fw[j]), b = __builtin_bit_cast(f32x4, fx[i]);
#pragma unroll
            for (int q = 0; q < 4; q++) acc[j][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[q], b[q], acc[j][i], 0, 0, 0);
          }
        }
    }
    if (kt + 1 < nk) stash(s ^ 1);
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < TM; i++) {
    int t = m0 + wm + i * 16 + fr;
    if (t >= n_tok) continue;
    float scale = 1.0f;
    if constexpr (BANK) {
      const int at = l.order[t];
      if (MODE == EPI_GLU || MODE == EPI_SPLIT) scale = l.scale[at]; else t = at;
    }
    if constexpr (MODE == EPI_GLU) {
#pragma unroll
      for (int j = 0; j < TN; j += 2) {
        const int n = n0 + wn + j * 16;                // block of 16 gate rows; its up rows are the next fragment
        if (n >= n_rows) continue;
        const int o = (n >> 1) + fc * 4;
        float v[4];
#pragma unroll
        for (int q = 0; q < 4; q++) v[q] = glu_pair(e.glu, e.limit, acc[j][i][q], acc[j + 1][i][q]);
        if constexpr (BANK) {
#pragma unroll
          for (int q = 0; q < 4; q++) v[q] *= scale;
        }
        put_four<AT>(e.h, (int64_t)t * e.ldh + o, f32x4{v[0], v[1], v[2], v[3]});
      }
      continue;
    }
    if constexpr (BANK && MODE == EPI_SPLIT) {           // (split 0, rows in whole fours)
#pragma unroll
      for (int j = 0; j < TN; j++) {
        const int n = n0 + wn + j * 16 + fc * 4;
        if (n >= n_rows) continue;
        put_four<AT>(e.h, (int64_t)t * e.ldh + n, lin_act_four(acc[j][i], e.act, e.limit) * scale);
      }
      continue;
    }
    const bool whole = (e.ldy & 3) == 0 && (e.ldh & 3) == 0 && (e.ld0 & 3) == 0 && (e.ldg & 3) == 0 && (e.split & 3) == 0;
#pragma unroll
    for (int j = 0; j < TN; j++) {
      const int n = n0 + wn + j * 16 + fc * 4;
      if (n >= n_rows) continue;
      if (n + 3 < n_rows && whole) epi_four<AT, MODE>(e, n, t, acc[j][i]);
      else {
#pragma unroll
        for (int q = 0; q < 4; q++) if (n + q < n_rows) epi_as<AT, MODE>(e, n + q, t, acc[j][i][q]);
      }
    }
  }
}

template <typename AT, int BM, int BN, int WM, int WN>
static void run_gemm(const cai_qw_s* w, const AT* x, int64_t ldx, int n_tok, const LinEpi& e)
{
  const int tm = (n_tok + BM - 1) / BM, tn = ((int)w->rows + BN - 1) / BN;
#define GEMM(MODE) case MODE: hipLaunchKernelGGL((gemm_bf16<AT, BM, BN, WM, WN, false, MODE>), dim3(tm * tn), dim3(64 * WM * WN), 0, ctx().stream, \
                              (const uint16_t*)w->data, x, (int)w->rows, (int)w->ld, ldx, n_tok, tm, tm * tn, e, BankList{}); break
  switch (e.mode) { GEMM(EPI_STORE); GEMM(EPI_GLU); GEMM(EPI_RESIDUAL); GEMM(EPI_SPLIT); GEMM(EPI_JOIN); }
#undef GEMM
}

template <typename AT, int BM, int BN>
static void run_bank(const cai_qw_s* w, int mat_rows, const AT* x, int64_t ldx, const BankList& l, const LinEpi& e)
{
  const int tm = l.max_tiles, tn = (mat_rows + BN - 1) / BN;
#define GEMM(MODE) case MODE: hipLaunchKernelGGL((gemm_bf16<AT, BM, BN, 2, 2, true, MODE>), dim3(tm * tn), dim3(256), 0, ctx().stream, \
                              (const uint16_t*)w->data, x, mat_rows, (int)w->ld, ldx, 0, tm, tm * tn, e, l); break
  switch (e.mode) { GEMM(EPI_STORE); GEMM(EPI_GLU); GEMM(EPI_SPLIT); }
#undef GEMM
}

int launch_lin_bank(const cai_qw_s* w, int mat_rows, int act_t, const void* x, int64_t ldx, const BankList& l, const LinEpi& e)
{
  CAI_REQUIRE(w->qtype == CAI_BF16 && mat_rows >= 1 && w->rows % mat_rows == 0 && ldx >= w->ld && l.max_tiles >= 1, "bf16 bank: matrices of %d rows of %lld, activation rows of %lld", mat_rows, (long long)w->rows, (long long)ldx);
  CAI_REQUIRE(e.mode == EPI_STORE || (e.mode == EPI_GLU && mat_rows % 32 == 0) || (e.mode == EPI_SPLIT && e.split == 0 && !e.bias && mat_rows % 4 == 0 && e.ldh % 4 == 0), "bf16 bank: a gated matrix needs whole blocks of 32 rows, another one of 4");
  CAI_REQUIRE(l.tile == BANK_TILE || l.tile == BANK_TILE_MAX, "bf16 bank: runs of %d places", l.tile);
  if (act_t == ACT_T_BF16) {
    if (l.tile == BANK_TILE_MAX) run_bank<bf16_t, BANK_TILE_MAX, 128>(w, mat_rows, (const bf16_t*)x, ldx, l, e);
    else run_bank<bf16_t, BANK_TILE, 64>(w, mat_rows, (const bf16_t*)x, ldx, l, e);
  } else if (l.tile == BANK_TILE_MAX) run_bank<float, BANK_TILE_MAX, 128>(w, mat_rows, (const float*)x, ldx, l, e);
  else run_bank<float, BANK_TILE, 64>(w, mat_rows, (const float*)x, ldx, l, e);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

// four rows a wave once that still leaves every CU eight waves; fewer rows, then a split of the row, for small matrices
struct GvShape { bool four; int ks; };
static GvShape gv_shape(int rows, int turns, bool glu)
{
  const int want = ctx().n_cu * 8;
  const bool four = rows / 4 >= want;
  const int groups = glu ? (four ? (rows / 2 + 1) / 2 : rows / 2) : (rows + (four ? 3 : 1)) / (four ? 4 : 2);
  int ks = 1;
  while (ks < GV_WAVES && ks * 2 <= turns && groups * ks * 2 <= want * 2) ks *= 2;
  return {four, ks};
}
static int gv_blocks(int rows, const GvShape& s, bool glu)
{
  const int groups = glu ? (s.four ? (rows / 2 + 1) / 2 : rows / 2) : (rows + (s.four ? 3 : 1)) / (s.four ? 4 : 2), per = GV_WAVES / s.ks;
  return (groups + per - 1) / per;
}
static int gv_turns(const cai_qw_s* w) { return ((int)w->ld + 511) / 512; }

template <typename AT, int NB, int KIND>
static void run_gemv(const cai_qw_s* w, const void* x, int64_t ldx, const LinEpi& e, const GvShape& s, int blocks, int turns, const GvSecond& q)
{
  const dim3 grid(blocks), blk(64 * GV_WAVES);
  const size_t lds = NB == 1 ? (size_t)std::min(GV_LDS, turns * 512) * 4 : 0;
  if (s.four) hipLaunchKernelGGL((gemv_bf16<AT, NB, 4, KIND>), grid, blk, lds, ctx().stream, (const uint16_t*)w->data, x, (int)w->rows, (int)w->ld, ldx, s.ks, e, q);
  else hipLaunchKernelGGL((gemv_bf16<AT, NB, 2, KIND>), grid, blk, lds, ctx().stream, (const uint16_t*)w->data, x, (int)w->rows, (int)w->ld, ldx, s.ks, e, q);
}
template <typename AT, int KIND>
static void run_gemv_rows(int n_tok, const cai_qw_s* w, const void* x, int64_t ldx, const LinEpi& e, const GvShape& s, int blocks, int turns, const GvSecond& q)
{
  switch (n_tok) {
    case 1: run_gemv<AT, 1, KIND>(w, x, ldx, e, s, blocks, turns, q); break;
    case 2: run_gemv<AT, 2, KIND>(w, x, ldx, e, s, blocks, turns, q); break;
    case 3: run_gemv<AT, 3, KIND>(w, x, ldx, e, s, blocks, turns, q); break;
    case 4: run_gemv<AT, 4, KIND>(w, x, ldx, e, s, blocks, turns, q); break;
    case 5: run_gemv<AT, 5, KIND>(w, x, ldx, e, s, blocks, turns, q); break;
    case 6: run_gemv<AT, 6, KIND>(w, x, ldx, e, s, blocks, turns, q); break;
    case 7: run_gemv<AT, 7, KIND>(w, x, ldx, e, s, blocks, turns, q); break;
    default: run_gemv<AT, 8, KIND>(w, x, ldx, e, s, blocks, turns, q); break;
  }
}

template <typename AT>
static int run_lin(const cai_qw_s* w, const AT* x, int64_t ldx, int n_tok, const LinEpi& e)
{
  if (n_tok <= LIN_FEW) {
    const bool glu = e.mode == EPI_GLU;
    const GvShape s = gv_shape((int)w->rows, gv_turns(w), glu);
    run_gemv_rows<AT, GV_PLAIN>(n_tok, w, x, ldx, e, s, gv_blocks((int)w->rows, s, glu), gv_turns(w), GvSecond());
    return CAI_OK;
  }
  auto tiles = [&](int bm, int bn) { return (int64_t)((n_tok + bm - 1) / bm) * ((w->rows + bn - 1) / bn); };
  if (n_tok > 64 && tiles(128, 128) >= ctx().n_cu) run_gemm<AT, 128, 128, 2, 2>(w, x, ldx, n_tok, e);
  else if (n_tok > 32 && tiles(64, 64) >= ctx().n_cu) run_gemm<AT, 64, 64, 2, 2>(w, x, ldx, n_tok, e);
  else run_gemm<AT, 32, 64, 2, 2>(w, x, ldx, n_tok, e);
  return CAI_OK;
}

int launch_lin_rms(int act_t, const float* x, int64_t ldx, int width, float eps, int n_tok, const RmsLin& a, const RmsLin* b)
{
  CAI_REQUIRE(n_tok >= 1 && n_tok <= LIN_FEW && a.w->cols == width && (!b || b->w->cols == width), "normed bf16 products: %d rows of %d columns", n_tok, width);
  auto mode_ok = [](const LinEpi& e) { return e.mode == EPI_STORE || e.mode == EPI_SPLIT; };
  CAI_REQUIRE(mode_ok(a.e) && (!b || mode_ok(b->e)), "normed bf16 products: an epilogue of another kind");
  CAI_REQUIRE(!b || !a.normed || !b->normed || a.ldn == b->ldn, "normed bf16 products: rows of two strides");
  const GvShape s = gv_shape((int)a.w->rows + (b ? (int)b->w->rows : 0), gv_turns(a.w), false);
  GvSecond q;
  q.blocks = gv_blocks((int)a.w->rows, s, false); q.width = width; q.eps = eps; q.gain = a.gain; q.normed = a.normed; q.ldn = a.ldn;
  int blocks = q.blocks;
  if (b) {
    q.W = (const uint16_t*)b->w->data; q.n_rows = (int)b->w->rows; q.e = b->e; q.gain2 = b->gain; q.normed2 = b->normed;
    if (b->normed) q.ldn = b->ldn;
    blocks += gv_blocks((int)b->w->rows, s, false);
  }
  if (act_t == ACT_T_BF16) run_gemv_rows<bf16_t, GV_RMS>(n_tok, a.w, x, ldx, a.e, s, blocks, gv_turns(a.w), q);
  else run_gemv_rows<float, GV_RMS>(n_tok, a.w, x, ldx, a.e, s, blocks, gv_turns(a.w), q);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int launch_lin_pair(int act_t, int n_tok, const cai_qw_s* w, const void* x, int64_t ldx, const LinEpi& e, const cai_qw_s* w2, const void* x2, int64_t ldx2, const LinEpi& e2)
{
  CAI_REQUIRE(n_tok >= 1 && n_tok <= LIN_FEW && w->rows == w2->rows && ldx >= w->ld && ldx2 >= w2->ld, "pair of bf16 products: %d rows, %lld and %lld outputs", n_tok, (long long)w->rows, (long long)w2->rows);
  CAI_REQUIRE(e.mode == EPI_JOIN && e2.mode == EPI_JOIN && e.y == e2.y && e.ldy == e2.ldy, "pair of bf16 products: both join one stream");
  const GvShape s = gv_shape((int)w->rows, std::min(gv_turns(w), gv_turns(w2)), false);
  GvSecond q;
  q.W = (const uint16_t*)w2->data; q.x = x2; q.ldw = (int)w2->ld; q.ldx = ldx2; q.e = e2;
  const int blocks = gv_blocks((int)w->rows, s, false), turns = std::max(gv_turns(w), gv_turns(w2));
  if (act_t == ACT_T_BF16) run_gemv_rows<bf16_t, GV_PAIR>(n_tok, w, x, ldx, e, s, blocks, turns, q);
  else run_gemv_rows<float, GV_PAIR>(n_tok, w, x, ldx, e, s, blocks, turns, q);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

int launch_lin(const cai_qw_s* w, int act_t, const void* x, int64_t ldx, int n_tok, const LinEpi& e)
{
  CAI_REQUIRE(w->qtype == CAI_BF16 && n_tok >= 1 && ldx >= w->ld, "bf16 linear layer: %lld columns need activation rows of %lld, got %lld", (long long)w->cols, (long long)w->ld, (long long)ldx);
  CAI_REQUIRE(e.mode != EPI_GLU || w->rows % 32 == 0, "bf16 linear layer: a gated matrix needs whole blocks of 32 rows");
  const int rc = act_t == ACT_T_BF16 ? run_lin<bf16_t>(w, (const bf16_t*)x, ldx, n_tok, e) : run_lin<float>(w, (const float*)x, ldx, n_tok, e);
  if (rc) return rc;
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

// ------------------------------------------------------------------------------------------
// float columns [col0, col0 + cols) of x -> padded activation rows of the chosen type
// ------------------------------------------------------------------------------------------
template <typename AT>
__global__ __launch_bounds__(256) void pack_rows_kernel(const float* x, int64_t ldx, int64_t col0, int cols, void* out, int64_t ldo)
{
  const int t = blockIdx.y;
  for (int i = blockIdx.x * 256 + threadIdx.x; i < ldo; i += gridDim.x * 256)
    put_act<AT>(out, t * ldo + i, i < cols ? x[t * ldx + col0 + i] : 0.0f);
}
int launch_pack_rows(const float* x, int64_t ldx, int64_t col0, int cols, int n_tok, int act_t, void* out, int64_t ldo)
{
  const dim3 grid((unsigned)std::min<int64_t>((ldo + 255) / 256, 32), n_tok);
  if (act_t == ACT_T_BF16) hipLaunchKernelGGL(pack_rows_kernel<bf16_t>, grid, dim3(256), 0, ctx().stream, x, ldx, col0, cols, out, ldo);
  else hipLaunchKernelGGL(pack_rows_kernel<float>, grid, dim3(256), 0, ctx().stream, x, ldx, col0, cols, out, ldo);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

__global__ __launch_bounds__(256) void bf16_rows_kernel(const uint16_t* w, int64_t ld, int64_t cols, int64_t row0, float* out)
{
  const int64_t r = blockIdx.y;
  for (int64_t i = blockIdx.x * 256 + threadIdx.x; i < cols; i += (int64_t)gridDim.x * 256)
    out[r * cols + i] = __builtin_bit_cast(float, (uint32_t)w[(row0 + r) * ld + i] << 16);
}
int bf16_dequant_rows(const cai_qw_s* w, int64_t row0, int64_t n_rows, float* out)
{
  for (int64_t r = 0; r < n_rows; r += 32768)
    hipLaunchKernelGGL(bf16_rows_kernel, dim3((unsigned)std::min<int64_t>((w->cols + 255) / 256, 32), (unsigned)std::min<int64_t>(n_rows - r, 32768)), dim3(256), 0, ctx().stream,
                       (const uint16_t*)w->data, w->ld, w->cols, row0 + r, out + r * w->cols);
  CAI_HIP(hipGetLastError());
  return CAI_OK;
}

// the stand-alone products (cai_qgemv, cai_qgemm) take unpadded float rows
static float* g_pack = nullptr; static size_t g_pack_cap = 0;
void bf16_release() { if (g_pack) (void)hipFree(g_pack); g_pack = nullptr; g_pack_cap = 0; }
int bf16_linear_f32(const cai_qw_s* w, const float* x, int64_t ldx, int n_tok, float* y, int64_t ldy, int act)
{
  const size_t need = (size_t)n_tok * w->ld;
  if (g_pack_cap < need) {
    CAI_HIP(hipStreamSynchronize(ctx().stream));
    bf16_release();
    CAI_HIP(hipMalloc((void**)&g_pack, need * 4));
    g_pack_cap = need;
  }
  int rc = launch_pack_rows(x, ldx, 0, (int)w->cols, n_tok, ACT_T_F32, g_pack, w->ld);
  if (rc) return rc;
  LinEpi e; e.y = y; e.ldy = ldy; e.bias = w->bias; e.act = act;
  return launch_lin(w, ACT_T_F32, g_pack, w->ld, n_tok, e);
}

}  // namespace cai
