// True 32-bit TN GEMM, Y[M, N] = X[M, K] W[N, K]^T (+ R), for the 32-bit mode of the
// models that have one.  64 x 64 tiles, 16-wide k-steps through LDS, 4 x 4
// outputs per thread with plain fp32 FMAs.  Every output is one sum in k order,
// so a row's result does not depend on the other rows of the call.
#include "common.h"
#include "kernels.h"

namespace {
constexpr int FT = 64, FK = 16;

__global__ __launch_bounds__(256) void gemm_f32_kernel(const float* __restrict__ X,
                                                       const float* __restrict__ W,
                                                       const float* __restrict__ R, float* __restrict__ Y, int M, int N, int K) {
  __shared__ float xs[FK][FT + 4], ws[FK][FT + 4];
  const int m0 = blockIdx.y * FT, n0 = blockIdx.x * FT;
  const int tr = threadIdx.x >> 4, tc = threadIdx.x & 15;
  const int lr = threadIdx.x >> 2, lk = (threadIdx.x & 3) * 4;
  const float* xp = X + (size_t)min(m0 + lr, M - 1) * K + lk;
  const float* wp = W + (size_t)min(n0 + lr, N - 1) * K + lk;
  float acc[4][4] = {};
  for (int k = 0; k < K; k += FK) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(xp + k);
    const f32x4 b = *reinterpret_cast<const f32x4*>(wp + k);
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      xs[lk + j][lr] = a[j];
      ws[lk + j][lr] = b[j];
    }
    __syncthreads();
#pragma unroll
    for (int q = 0; q < FK; ++q) {
      const f32x4 av = *reinterpret_cast<const f32x4*>(&xs[q][tr * 4]);
      const f32x4 bv = *reinterpret_cast<const f32x4*>(&ws[q][tc * 4]);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(av[i], bv[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = m0 + tr * 4 + i, n = n0 + tc * 4;
    if (m < M && n < N) {
      f32x4 v = f32x4{acc[i][0], acc[i][1], acc[i][2], acc[i][3]};
      if (R) v += *reinterpret_cast<const f32x4*>(R + (size_t)m * N + n);
      *reinterpret_cast<f32x4*>(Y + (size_t)m * N + n) = v;
    }
  }
}

// gated activation of the 32-bit mode: g | u rows interleaved in 16-row groups
// as for the fused bf16 epilogues; y = act(g) u
__global__ __launch_bounds__(256) void gated_act_f32_kernel(const float* __restrict__ z,
                                                            float* __restrict__ y, int M, int F,
                                                            int act) {
  const size_t total = (size_t)M * F;
  for (size_t i = blockIdx.x * 256ull + threadIdx.x; i < total; i += (size_t)gridDim.x * 256) {
    const size_t m = i / F;
    const int f = (int)(i % F);
    const float* p = z + m * 2 * F + (f >> 4) * 32 + (f & 15);
    const float g = p[0], u = p[16];
    float a;
    if (act == ACT_GELU_TANH)
      a = 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
    else
      a = g / (1.f + expf(-g));
    y[i] = a * u;
  }
}
}  // namespace

int launch_gemm_f32(const float* X, const float* W, const float* R, float* Y, int M, int N, int K,
                    hipStream_t s) {
  if (K % FK || N % 4) return 1;
  if (M <= 0 || N <= 0) return 0;
  gemm_f32_kernel<<<dim3((N + FT - 1) / FT, (M + FT - 1) / FT), 256, 0, s>>>(X, W, R, Y, M, N, K);
  return 0;
}

void launch_gated_act_f32(const float* z, float* y, int M, int F, int act, hipStream_t s) {
  const size_t n = (size_t)M * F;
  if (!n) return;
  const size_t g = (n + 255) / 256;
  gated_act_f32_kernel<<<(unsigned)(g > 4096 ? 4096 : g), 256, 0, s>>>(z, y, M, F, act);
}
