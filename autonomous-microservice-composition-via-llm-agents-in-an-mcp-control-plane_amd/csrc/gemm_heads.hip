// One product per head, out[t, h, :] = X[t, h, :] W[h]^T: the absorbed key and
// value projections of latent attention.  X and out are strided [T, H, .] views,
// W [H, N, K].  MFMA accumulators hold out^T (A = W rows, B = X rows), so a lane
// owns four neighbouring outputs of one token.  Three forms:
//   few   up to 64 tokens (decode): a block per 16 outputs of a head, the sum over
//         k shared out to its 4 waves, operands straight from global memory;
//   tile  128 tokens x 128 outputs per block, LDS-DMA staging, stores through
//         LDS so that a token's outputs leave as whole lines;
//   f32   the 32-bit mode, plain FMAs, one sum in k order per output.
#include "common.h"
#include "kernels.h"

namespace {

// ------------------------------------------------------------------ few tokens
template <int NT>
__global__ __launch_bounds__(256) void heads_few_kernel(const HeadGemmArgs a) {
  __shared__ f32x4 part[4][NT][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int fr = lane & 15, fq = lane >> 4;
  const int h = blockIdx.y, n0 = blockIdx.x * 16;
  const bf16* w = (const bf16*)a.W + ((size_t)h * a.N + n0 + fr) * a.K + 8 * fq;
  const bf16* x[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i)
    x[i] = (const bf16*)a.X + (size_t)min(i * 16 + fr, a.T - 1) * a.xt + (size_t)h * a.xh + 8 * fq;
  f32x4 acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = wave * 32; k < a.K; k += 128) {
    const bf16x8 wf = *reinterpret_cast<const bf16x8*>(w + k);
#pragma unroll
    for (int i = 0; i < NT; ++i)
      acc[i] = mfma16x16x32(wf, *reinterpret_cast<const bf16x8*>(x[i] + k), acc[i]);
  }
#pragma unroll
  for (int i = 0; i < NT; ++i) part[wave][i][lane] = acc[i];
  __syncthreads();
  const int t = wave * 16 + fr;                         // wave i adds token tile i
  if (wave >= NT || t >= a.T) return;
  const f32x4 v = part[0][wave][lane] + part[1][wave][lane] + part[2][wave][lane] + part[3][wave][lane];
  bf16x4 o;
#pragma unroll
  for (int r = 0; r < 4; ++r) o[r] = (bf16)v[r];
  *reinterpret_cast<bf16x4*>((bf16*)a.out + (size_t)t * a.ot + (size_t)h * a.oh + n0 + 4 * fq) = o;
}

// ------------------------------------------------------------------------ tile
constexpr int TM = 128, TN = 128;             // tokens x outputs of a block

// LDS-DMA of [128][BK] of rows at ``src`` (row stride ld, rows from ``rows`` on
// repeat the last one), 16-B chunks swizzled by row
template <int BK>
DEV void stage_tile(const bf16* src, long long ld, int rows, bf16* dst, int wave, int lane) {
  constexpr int NC = BK / 8, PW = TM * NC / 64 / 4;     // chunks per row, pieces per wave
#pragma unroll
  for (int i = 0; i < PW; ++i) {
    const int p = wave * PW + i, c = p * 64 + lane;
    const int row = c / NC, chunk = c % NC;
    glds16(src + (size_t)min(row, rows - 1) * ld + ((chunk ^ (row & (NC - 1))) << 3), dst + p * 512);
  }
}

template <int BK>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2))) void heads_tile_kernel(
    const HeadGemmArgs a) {
  constexpr int NC = BK / 8;
  constexpr int OLD = TN + 8;                           // LDS row of the staged output
  constexpr int STAGE = 2 * (TM + TN) * BK, OUT = TM * OLD;
  __shared__ __attribute__((aligned(16))) bf16 smem[STAGE > OUT ? STAGE : OUT];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int fr = lane & 15, fq = lane >> 4;
  const int h = blockIdx.z, t0 = blockIdx.y * TM, n0 = blockIdx.x * TN;
  const int rt = min(a.T - t0, TM), rn = min(a.N - n0, TN);
  const bf16* X = (const bf16*)a.X + (size_t)t0 * a.xt + (size_t)h * a.xh;
  const bf16* W = (const bf16*)a.W + ((size_t)h * a.N + n0) * a.K;
  const int wt = (wave & 1) * 64, wn = (wave >> 1) * 64;
  f32x4 acc[4][4];                                      // [outputs][tokens], 16 x 16 each
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int steps = a.K / BK;
  auto stage = [&](int k) {
    bf16* b = smem + (k & 1) * (TM + TN) * BK;
    stage_tile<BK>(X + k * BK, a.xt, rt, b, wave, lane);
    stage_tile<BK>(W + k * BK, a.K, rn, b + TM * BK, wave, lane);
  };
  stage(0);
  for (int k = 0; k < steps; ++k) {
    __syncthreads();                                    // tile k is in LDS, the other buffer is free
    if (k + 1 < steps) stage(k + 1);
    const bf16* Xl = smem + (k & 1) * (TM + TN) * BK;
    const bf16* Wl = Xl + TM * BK;
#pragma unroll
    for (int ks = 0; ks < BK / 32; ++ks) {
      bf16x8 wf[4], xf[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int rw = wn + i * 16 + fr, rx = wt + i * 16 + fr;
        wf[i] = *reinterpret_cast<const bf16x8*>(Wl + rw * BK + (((ks * 4 + fq) ^ (rw & (NC - 1))) << 3));
        xf[i] = *reinterpret_cast<const bf16x8*>(Xl + rx * BK + (((ks * 4 + fq) ^ (rx & (NC - 1))) << 3));
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mfma16x16x32(wf[i], xf[j], acc[i][j]);
    }
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      bf16x4 o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = (bf16)acc[i][j][r];
      *reinterpret_cast<bf16x4*>(smem + (wt + j * 16 + fr) * OLD + wn + i * 16 + 4 * fq) = o;
    }
  __syncthreads();
  const int c = (threadIdx.x & 15) * 8;
  if (c >= rn) return;
  for (int r = threadIdx.x >> 4; r < rt; r += 16)
    *reinterpret_cast<bf16x8*>((bf16*)a.out + (size_t)(t0 + r) * a.ot + (size_t)h * a.oh + n0 + c) =
        *reinterpret_cast<const bf16x8*>(smem + r * OLD + c);
}

// ------------------------------------------------------------------- 32-bit
__global__ __launch_bounds__(256) void heads_f32_kernel(const HeadGemmArgs a) {
  constexpr int FT = 64, FK = 16;
  __shared__ float xs[FK][FT + 4], ws[FK][FT + 4];
  const int h = blockIdx.z, t0 = blockIdx.y * FT, n0 = blockIdx.x * FT;
  const int tr = threadIdx.x >> 4, tc = threadIdx.x & 15;
  const int lr = threadIdx.x >> 2, lk = (threadIdx.x & 3) * 4;
  const float* xp = (const float*)a.X + (size_t)min(t0 + lr, a.T - 1) * a.xt + (size_t)h * a.xh + lk;
  const float* wp = (const float*)a.W + ((size_t)h * a.N + min(n0 + lr, a.N - 1)) * a.K + lk;
  float acc[4][4] = {};
  for (int k = 0; k < a.K; k += FK) {
    const f32x4 x = *reinterpret_cast<const f32x4*>(xp + k);
    const f32x4 w = *reinterpret_cast<const f32x4*>(wp + k);
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      xs[lk + j][lr] = x[j];
      ws[lk + j][lr] = w[j];
    }
    __syncthreads();
#pragma unroll
    for (int q = 0; q < FK; ++q) {
      const f32x4 xv = *reinterpret_cast<const f32x4*>(&xs[q][tr * 4]);
      const f32x4 wv = *reinterpret_cast<const f32x4*>(&ws[q][tc * 4]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xv[i], wv[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = t0 + tr * 4 + i, n = n0 + tc * 4;
    if (t < a.T && n < a.N)
      *reinterpret_cast<f32x4*>((float*)a.out + (size_t)t * a.ot + (size_t)h * a.oh + n) =
          f32x4{acc[i][0], acc[i][1], acc[i][2], acc[i][3]};
  }
}

}  // namespace

int launch_gemm_heads(const HeadGemmArgs& a, bool f32, hipStream_t s) {
  if (a.K % 32 || a.N % 16 || a.xt % 8 || a.xh % 8 || a.ot % 8 || a.oh % 8) return 1;
  if (a.T <= 0) return 0;
  if (f32) {
    heads_f32_kernel<<<dim3((a.N + 63) / 64, (a.T + 63) / 64, a.H), 256, 0, s>>>(a);
    return 0;
  }
  if (a.T <= 64) {
    const dim3 grid(a.N / 16, a.H);
    if (a.T <= 16) heads_few_kernel<1><<<grid, 256, 0, s>>>(a);
    else if (a.T <= 32) heads_few_kernel<2><<<grid, 256, 0, s>>>(a);
    else heads_few_kernel<4><<<grid, 256, 0, s>>>(a);
    return 0;
  }
  const dim3 grid((a.N + TN - 1) / TN, (a.T + TM - 1) / TM, a.H);
  if (a.K % 64) heads_tile_kernel<32><<<grid, 256, 0, s>>>(a);
  else heads_tile_kernel<64><<<grid, 256, 0, s>>>(a);
  return 0;
}
