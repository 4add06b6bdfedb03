// Projected rows -> queries and paged cache, for attention whose heads are normed
// after the projection and for latent attention.  T is bf16, or float in the
// 32-bit mode; norms, rotation and value mixing are fp32.
#include "rows.h"
#include "kernels.h"

namespace {

// ---- rms norm of every q / k head, value mixing, cache write.  LG lanes per
// (token, head), 8 elements a lane and step, at most NCH steps.
template <class T, int LG, int NCH>
__global__ __launch_bounds__(256) void qk_norm_kv_kernel(
    const T* __restrict__ z, int ldz, const int* __restrict__ slots, const float* __restrict__ wq,
    const float* __restrict__ wk, float inv_dim, float eps, T* __restrict__ q_out,
    T* __restrict__ k_cache, T* __restrict__ v_cache, const T* __restrict__ v_first, int ldv,
    float lam, int T_, int Hq, int Hkv, int DK, int DV, int BS) {
  const int per = Hq + 2 * Hkv, li = threadIdx.x % LG;
  const size_t unit = (blockIdx.x * 256ull + threadIdx.x) / LG;
  if (unit >= (size_t)T_ * per) return;                  // (whole groups of LG lanes)
  const int t = (int)(unit / per), u = (int)(unit % per);
  const bool is_v = u >= Hq + Hkv, is_q = u < Hq;
  const int h = is_q ? u : is_v ? u - Hq - Hkv : u - Hq;
  const int nv = (is_v ? DV : DK) / 8;
  const T* src = z + (size_t)t * ldz + (is_v ? (Hq + Hkv) * DK + h * DV : u * DK);
  const int slot = is_q ? 0 : slots[t];
  T* dst;
  if (is_q) {
    dst = q_out + ((size_t)t * Hq + h) * DK;
  } else {
    const size_t row = ((size_t)(max(slot, 0) / BS) * Hkv + h) * BS + max(slot, 0) % BS;
    dst = is_v ? v_cache + row * DV : k_cache + row * DK;
  }
  float v[NCH][8];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NCH; ++i) {
    const int c = li + i * LG;
    if (c < nv) {
      load8(src + c * 8, v[i]);
#pragma unroll
      for (int j = 0; j < 8; ++j) ss = fmaf(v[i][j], v[i][j], ss);
    }
  }
#pragma unroll
  for (int o = LG / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  if (slot < 0) return;
  const float inv = 1.f / sqrtf(ss * inv_dim + eps);
  const float* w = is_q ? wq : wk;
#pragma unroll
  for (int i = 0; i < NCH; ++i) {
    const int c = li + i * LG;
    if (c >= nv) continue;
    if (!is_v) {
      float g[8];
      load8(w + c * 8, g);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[i][j] = v[i][j] * inv * g[j];
    } else if (v_first) {
      float f[8];
      load8(v_first + (size_t)t * ldv + h * DV + c * 8, f);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[i][j] = (1.f - lam) * v[i][j] + lam * f[j];
    }
    store8(dst + c * 8, v[i]);
  }
}

template <class T>
int qk_norm_kv_dispatch(const T* z, int ldz, const int* slots, const float* wq, const float* wk,
                        int dim, float eps, T* q_out, T* k_cache, T* v_cache, const T* v_first,
                        int ldv, float lam, int T_, int Hq, int Hkv, int DK, int DV, int BS,
                        hipStream_t s) {
#define QKN(LG, NCH)                                                                               \
  {                                                                                                \
    const size_t groups = (size_t)T_ * (Hq + 2 * Hkv);                                             \
    qk_norm_kv_kernel<T, LG, NCH><<<(unsigned)((groups * LG + 255) / 256), 256, 0, s>>>(           \
        z, ldz, slots, wq, wk, 1.f / (float)dim, eps, q_out, k_cache, v_cache, v_first, ldv, lam,  \
        T_, Hq, Hkv, DK, DV, BS);                                                                  \
    return 0;                                                                                      \
  }
  const int n = (DK > DV ? DK : DV) / 8;
  if (n <= 8) QKN(8, 1)
  if (n <= 16) QKN(16, 1)
  if (n <= 32) QKN(32, 1)
  if (n <= 64) QKN(64, 1)
  if (n <= 128) QKN(64, 2)
  return 1;
#undef QKN
}

// ---- latent attention: the token's cached row [rms(latent) w_c | rotated key |
// 0] and the queries' rotated parts.  One block per token; wave 0 takes the row,
// the others the heads.
template <class T>
__global__ __launch_bounds__(256) void latent_rows_kernel(const LatentRowArgs a) {
  const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const T* z = (const T*)a.z + (size_t)t * a.ldz;
  const float* cs = a.cos_sin + (size_t)a.pos[t] * a.pairs * 2;
  const int qs = a.dim + a.rot, tail = (a.DK - a.rank) / 8;
  if (wave) {
    if (!a.q_out) return;
    for (int i = threadIdx.x - 64; i < a.heads * tail; i += 192) {
      const int h = i / tail, d = (i % tail) * 8;
      float v[8];
      rotated8(z + h * qs + a.dim, cs, a.pairs, a.rot, d, v);
      store8((T*)a.q_out + ((size_t)t * a.heads + h) * a.DK + a.rank + d, v);
    }
    return;
  }
  const int slot = a.slots[t];
  if (slot < 0) return;
  T* row = (T*)a.k_cache + ((size_t)(slot / a.BS) * a.BS + slot % a.BS) * a.DK;
  const T* c = z + a.heads * qs;
  float ss = 0.f;
  for (int d = lane * 8; d < a.rank; d += 512) {
    float v[8];
    load8(c + d, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) ss = fmaf(v[j], v[j], ss);
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / (float)a.rank_true + a.eps);
  for (int d = lane * 8; d < a.rank; d += 512) {
    float v[8], w[8];
    load8(c + d, v);
    load8(a.w_c + d, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = v[j] * inv * w[j];
    store8(row + d, v);
  }
  for (int i = lane; i < tail; i += 64) {
    float v[8];
    rotated8(c + a.rank, cs, a.pairs, a.rot, i * 8, v);
    store8(row + a.rank + i * 8, v);
  }
}

// the latents of cached pages as plain rows: out [pages * BS, ldo], columns from
// ``rank`` on and rows from a page's ``valid`` on zero
__global__ __launch_bounds__(256) void latent_gather_kernel(const bf16* __restrict__ cache,
                                                            const int* __restrict__ pages,
                                                            const int* __restrict__ valid, int DK, int BS,
                                                            int rank, bf16* __restrict__ out, int ldo) {
  const int nc = ldo / 8, page = pages[blockIdx.x], n = valid[blockIdx.x];
  for (int i = threadIdx.x; i < BS * nc; i += 256) {
    const int r = i / nc, c = (i % nc) * 8;
    bf16x8 v = {};
    if (r < n && c < rank) v = *reinterpret_cast<const bf16x8*>(cache + ((size_t)page * BS + r) * DK + c);
    *reinterpret_cast<bf16x8*>(out + ((size_t)blockIdx.x * BS + r) * ldo + c) = v;
  }
}

}  // namespace

int launch_latent_gather(const void* cache, const int* pages, const int* valid, int n, int DK, int BS,
                         int rank, void* out, int ldo, hipStream_t s) {
  if (n <= 0) return 0;
  if (DK % 8 || rank % 8 || ldo % 8 || rank > DK || rank > ldo) return 1;
  latent_gather_kernel<<<n, 256, 0, s>>>((const bf16*)cache, pages, valid, DK, BS, rank, (bf16*)out, ldo);
  return 0;
}

int launch_qk_norm_kv(const void* z, int ldz, const int* slots, const float* wq, const float* wk,
                      int dim, float eps, void* q_out, void* k_cache, void* v_cache,
                      const void* v_first, int ldv, float lam, int T, int Hq, int Hkv, int DK,
                      int DV, int BS, bool f32, hipStream_t s) {
  if (T <= 0) return 0;
  if (DK % 8 || DV % 8 || ldz % 8 || ldv % 8) return 1;
  if (f32)
    return qk_norm_kv_dispatch<float>((const float*)z, ldz, slots, wq, wk, dim, eps, (float*)q_out,
                                      (float*)k_cache, (float*)v_cache, (const float*)v_first, ldv,
                                      lam, T, Hq, Hkv, DK, DV, BS, s);
  return qk_norm_kv_dispatch<bf16>((const bf16*)z, ldz, slots, wq, wk, dim, eps, (bf16*)q_out,
                                   (bf16*)k_cache, (bf16*)v_cache, (const bf16*)v_first, ldv, lam, T,
                                   Hq, Hkv, DK, DV, BS, s);
}

int launch_latent_rows(const LatentRowArgs& a, bool f32, hipStream_t s) {
  if (a.T <= 0) return 0;
  if (a.dim % 8 || a.rot % 8 || a.rank % 8 || a.DK % 8 || a.ldz % 8 || a.rank + a.rot > a.DK ||
      2 * a.pairs > a.rot)
    return 1;
  if (f32)
    latent_rows_kernel<float><<<a.T, 256, 0, s>>>(a);
  else
    latent_rows_kernel<bf16><<<a.T, 256, 0, s>>>(a);
  return 0;
}
