// Row kernels of decoders whose residual stream is fp32: the scaled embedding,
// the residual add (post-normed or plain) + next pre-norm (rms or layer norm) in
// one pass, and the capped logits.  T is the activation type of the projections (bf16, or float in the
// 32-bit mode); the residual, the norms and the logits are always fp32.
#include "common.h"
#include "kernels.h"

namespace {

template <class T>
struct Vec4;
template <>
struct Vec4<bf16> {
  typedef bf16x4 type;
};
template <>
struct Vec4<float> {
  typedef f32x4 type;
};

template <class T>
DEV f32x4 load4(const T* p) {
  const typename Vec4<T>::type v = *reinterpret_cast<const typename Vec4<T>::type*>(p);
  return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
}
template <class T>
DEV void store4(T* p, const f32x4& v) {
  typename Vec4<T>::type o;
#pragma unroll
  for (int j = 0; j < 4; ++j) o[j] = (T)v[j];
  *reinterpret_cast<typename Vec4<T>::type*>(p) = o;
}

template <int NT>
DEV float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
#pragma unroll
  for (int w = 0; w < NT / 64; ++w) t += red[w];
  return t;
}

// One block per row (1024 threads for few rows: shorter chains; 256 otherwise),
// 4 floats per thread and step, the row and the norm weights in registers
// between the passes:
//   y given:      x += y / rms(y) * w_post, or x += y   (written back)
//   w_pre given:  out = x / rms(x) * w_pre,  else out = x   (as T, row stride ld)
//   CENTER:       the row's mean comes off x before that norm (layer norm)
// Rows are Hp wide (columns >= H are zero and stay zero), means are over H.
template <class T, int VMAX, int NT, bool CENTER>
__global__ __launch_bounds__(NT) void residual_norm_kernel(
    float* __restrict__ x, const T* __restrict__ y, const float* __restrict__ w_post,
    const float* __restrict__ w_pre, T* __restrict__ out, int ld, int H, int Hp, float eps) {
  __shared__ float red[3][NT / 64];
  const int row = blockIdx.x, nvec = Hp >> 2;
  float* xr = x + (size_t)row * Hp;
  const float inv_h = 1.f / (float)H;
  constexpr bool EARLY = VMAX <= 2;                  // weights fit the registers too
  f32x4 xv[VMAX], yv[VMAX], wa[EARLY ? VMAX : 1], wb[EARLY ? VMAX : 1];
#pragma unroll
  for (int i = 0; i < VMAX; ++i) {
    const int c = threadIdx.x + i * NT;
    xv[i] = yv[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c < nvec) {
      xv[i] = *reinterpret_cast<const f32x4*>(xr + 4 * c);
      if (y) yv[i] = load4(y + (size_t)row * Hp + 4 * c);
      if constexpr (EARLY) {
        if (w_post) wa[i] = *reinterpret_cast<const f32x4*>(w_post + 4 * c);
        if (w_pre) wb[i] = *reinterpret_cast<const f32x4*>(w_pre + 4 * c);
      }
    }
  }
  if (y && !w_post) {
#pragma unroll
    for (int i = 0; i < VMAX; ++i) {
      const int c = threadIdx.x + i * NT;
      if (c < nvec) {
        xv[i] += yv[i];
        *reinterpret_cast<f32x4*>(xr + 4 * c) = xv[i];
      }
    }
  } else if (y) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VMAX; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) ss += yv[i][j] * yv[i][j];
    const float inv = 1.f / sqrtf(block_sum<NT>(ss, red[0]) * inv_h + eps);
#pragma unroll
    for (int i = 0; i < VMAX; ++i) {
      const int c = threadIdx.x + i * NT;
      if (c < nvec) {
        const f32x4 w = EARLY ? wa[EARLY ? i : 0] : *reinterpret_cast<const f32x4*>(w_post + 4 * c);
#pragma unroll
        for (int j = 0; j < 4; ++j) xv[i][j] += yv[i][j] * inv * w[j];
        *reinterpret_cast<f32x4*>(xr + 4 * c) = xv[i];
      }
    }
  }
  if (!out) return;
  float inv = 1.f;
  if (w_pre) {
    float ss = 0.f;
    if constexpr (CENTER) {
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < VMAX; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) sum += xv[i][j];
      const float mean = block_sum<NT>(sum, red[2]) * inv_h;
#pragma unroll
      for (int i = 0; i < VMAX; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)                    // (columns from H on stay zero)
          xv[i][j] = 4 * ((int)threadIdx.x + i * NT) + j < H ? xv[i][j] - mean : 0.f;
    }
#pragma unroll
    for (int i = 0; i < VMAX; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) ss += xv[i][j] * xv[i][j];
    inv = 1.f / sqrtf(block_sum<NT>(ss, red[1]) * inv_h + eps);
  }
  T* orow = out + (size_t)row * ld;
#pragma unroll
  for (int i = 0; i < VMAX; ++i) {
    const int c = threadIdx.x + i * NT;
    if (c < nvec) {
      f32x4 o = xv[i];
      if (w_pre) {
        const f32x4 w = EARLY ? wb[EARLY ? i : 0] : *reinterpret_cast<const f32x4*>(w_pre + 4 * c);
#pragma unroll
        for (int j = 0; j < 4; ++j) o[j] = o[j] * inv * w[j];
      }
      store4(orow + 4 * c, o);
    }
  }
}

template <class T>
void residual_norm_dispatch(float* x, const T* y, const float* w_post, const float* w_pre, T* out,
                            int ld, int rows, int H, int Hp, float eps, bool center, hipStream_t s) {
#define RN_CASE(V, NT)                                                                                     \
  (center ? residual_norm_kernel<T, V, NT, true><<<rows, NT, 0, s>>>(x, y, w_post, w_pre, out, ld, H, Hp, eps) \
          : residual_norm_kernel<T, V, NT, false><<<rows, NT, 0, s>>>(x, y, w_post, w_pre, out, ld, H, Hp, eps))
  if (rows <= 512 && Hp > 1024) {
    const int v = (Hp / 4 + 1023) / 1024;
    if (v <= 1) RN_CASE(1, 1024);
    else if (v <= 2) RN_CASE(2, 1024);
    else RN_CASE(4, 1024);
    return;
  }
  const int v = (Hp / 4 + 255) / 256;
  if (v <= 1) RN_CASE(1, 256);
  else if (v <= 2) RN_CASE(2, 256);
  else if (v <= 4) RN_CASE(4, 256);
  else if (v <= 8) RN_CASE(8, 256);
  else RN_CASE(16, 256);
#undef RN_CASE
}

// x[t] = table[ids[t]] * scale (fp32), and the same row as T into lo (row
// stride ld; null: not kept)
template <class T>
__global__ __launch_bounds__(256) void embedding_scaled_kernel(
    const int* __restrict__ ids, const T* __restrict__ table, float scale, float* __restrict__ x,
    T* __restrict__ lo, int ld, int Hp) {
  const int t = blockIdx.x;
  const T* src = table + (size_t)ids[t] * Hp;
  for (int c = threadIdx.x; c < (Hp >> 2); c += 256) {
    f32x4 v = load4(src + 4 * c);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] *= scale;
    *reinterpret_cast<f32x4*>(x + (size_t)t * Hp + 4 * c) = v;
    if (lo) store4(lo + (size_t)t * ld + 4 * c, v);
  }
}

// z <- cap tanh(z scale / cap) in place (cap 0: z scale)
__global__ __launch_bounds__(256) void logit_finish_kernel(float* __restrict__ z, size_t n,
                                                           float scale, float cap) {
  const float inv = cap > 0.f ? 1.f / cap : 0.f;
  for (size_t i = blockIdx.x * 256ull + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) {
    const float v = z[i] * scale;
    z[i] = cap > 0.f ? cap * tanhf(v * inv) : v;
  }
}

}  // namespace

int launch_residual_norm(float* x, const void* y, const float* w_post, const float* w_pre,
                         void* out, int ld, int rows, int H, int Hp, float eps, bool center,
                         bool f32, hipStream_t s) {
  if (rows <= 0) return 0;
  if (Hp % 4 || Hp > RESIDUAL_MAX_WIDTH || H > Hp || (w_post && !y)) return 1;
  if (f32)
    residual_norm_dispatch<float>(x, (const float*)y, w_post, w_pre, (float*)out, ld, rows, H, Hp, eps, center, s);
  else
    residual_norm_dispatch<bf16>(x, (const bf16*)y, w_post, w_pre, (bf16*)out, ld, rows, H, Hp, eps, center, s);
  return 0;
}

void launch_embedding_scaled(const int* ids, const void* table, float scale, float* x, void* lo,
                             int ld, int T, int Hp, bool f32, hipStream_t s) {
  if (T <= 0) return;
  if (f32)
    embedding_scaled_kernel<float><<<T, 256, 0, s>>>(ids, (const float*)table, scale, x, (float*)lo, ld, Hp);
  else
    embedding_scaled_kernel<bf16><<<T, 256, 0, s>>>(ids, (const bf16*)table, scale, x, (bf16*)lo, ld, Hp);
}

void launch_logit_finish(float* z, size_t n, float scale, float cap, hipStream_t s) {
  if (!n || (scale == 1.f && cap <= 0.f)) return;
  const size_t g = (n + 255) / 256;
  logit_finish_kernel<<<(unsigned)(g > 8192 ? 8192 : g), 256, 0, s>>>(z, n, scale, cap);
}
