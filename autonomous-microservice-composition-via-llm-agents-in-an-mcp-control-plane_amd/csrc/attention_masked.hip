// Paged attention with a mask and a softmax of a model's own choosing: logit
// soft-capping (s <- cap tanh(s / cap)), chunked causal masks (a query sees the
// keys of its own chunk of the sequence only), a sink of score 0 in the softmax
// denominator, key and value heads of different sizes, any GQA group.  The
// plain causal softmax kernels for d = 128 are in attention.hip.
//
// Layouts: q [T, Hq, DK], k cache [num_blocks, Hkv, 64, DK], v cache
// [num_blocks, Hkv, 64, DV], out [T, Hq, DV].
#include "common.h"
#include "kernels.h"

namespace {

constexpr int KT = 64;                        // keys per cache block

DEV int chunk_start(int pos, int chunk) { return chunk > 0 ? pos / chunk * chunk : 0; }

// ---- row form: one wave per (token, query head).  Lanes take keys for the
// scores and value columns for the sum; everything is fp32.  The 32-bit mode
// runs on it, and head sizes the MFMA forms do not cover.
constexpr int ROW_MAX_DV = 512;

template <class T>
__global__ __launch_bounds__(64) void attn_row_kernel(const MaskedAttnArgs a) {
  extern __shared__ float lds[];              // q row [DK], weights [64]
  float* qs = lds;
  float* ps = lds + a.DK;
  const int t = blockIdx.x, head = blockIdx.y, lane = threadIdx.x;
  const int kvh = head / (a.Hq / a.Hkv);
  int s = -1;
  for (int b = 0; b < a.S; b += 64) {         // the sequence that holds token t
    const int i = b + lane;
    const bool hit = i < a.S && t >= a.q_start[i] && t < a.q_start[i] + a.q_len[i];
    const unsigned long long m = __ballot(hit);
    if (m) {
      s = b + __ffsll(m) - 1;
      break;
    }
  }
  if (s < 0) return;
  const T* qp = (const T*)a.q + ((size_t)t * a.Hq + head) * a.DK;
  for (int d = lane; d < a.DK; d += 64) qs[d] = (float)qp[d];
  __syncthreads();
  const int qpos = a.ctx_len[s] - a.q_len[s] + (t - a.q_start[s]);
  const int first = chunk_start(qpos, a.chunk);
  const int* bt = a.block_table + (size_t)s * a.max_blocks;
  float m_run = a.sink ? 0.f : -INFINITY, l = a.sink ? 1.f : 0.f;
  float o[ROW_MAX_DV / 64];
#pragma unroll
  for (int i = 0; i < ROW_MAX_DV / 64; ++i) o[i] = 0.f;
  for (int kt = first / KT; kt <= qpos / KT; ++kt) {
    const size_t blk = (size_t)bt[kt] * a.Hkv + kvh;
    const T* kr = (const T*)a.kc + (blk * KT + lane) * a.DK;
    const int key = kt * KT + lane;
    const bool on = key >= first && key <= qpos;
    float sc = 0.f;
    if (on) {
      for (int d = 0; d < a.DK; ++d) sc = fmaf(qs[d], (float)kr[d], sc);
      sc *= a.scale;
      if (a.cap > 0.f) sc = a.cap * tanhf(sc / a.cap);
    }
    const float mt = wave_max(on ? sc : -INFINITY);
    const float m_new = fmaxf(m_run, mt);
    const float alpha = expf(m_run - m_new);
    const float p = on ? expf(sc - m_new) : 0.f;
    m_run = m_new;
    l = l * alpha + wave_sum(p);
    __syncthreads();
    ps[lane] = p;
    __syncthreads();
    const int k0 = max(first - kt * KT, 0), k1 = min(qpos - kt * KT, KT - 1);
#pragma unroll
    for (int i = 0; i < ROW_MAX_DV / 64; ++i) {
      const int d = i * 64 + lane;
      if (d < a.DV) {
        float acc = o[i] * alpha;
        const T* vr = (const T*)a.vc + blk * KT * a.DV + d;
        for (int k = k0; k <= k1; ++k) acc = fmaf(ps[k], (float)vr[(size_t)k * a.DV], acc);
        o[i] = acc;
      }
    }
  }
  const float inv = 1.f / l;
  T* op = (T*)a.out + ((size_t)t * a.Hq + head) * a.DV;
#pragma unroll
  for (int i = 0; i < ROW_MAX_DV / 64; ++i) {
    const int d = i * 64 + lane;
    if (d < a.DV) op[d] = (T)(o[i] * inv);
  }
}

}  // namespace

int launch_attn_row(const MaskedAttnArgs& a, int T, bool f32, hipStream_t s) {
  if (T <= 0) return 0;
  if (a.DV > ROW_MAX_DV || a.Hq % a.Hkv) return 1;
  const size_t lds = (size_t)(a.DK + 64) * sizeof(float);
  if (f32)
    attn_row_kernel<float><<<dim3(T, a.Hq), 64, lds, s>>>(a);
  else
    attn_row_kernel<bf16><<<dim3(T, a.Hq), 64, lds, s>>>(a);
  return 0;
}
