// Paged attention with a mask and a softmax of a model's own choosing: logit
// soft-capping (s <- cap tanh(s / cap)), chunked causal masks (a query sees the
// keys of its own chunk of the sequence only), sliding windows that keep the
// first keys, scores that fall with the distance, a sink in the softmax
// denominator (of score 0 or learned), a gate on every head's output, key and
// value heads of different sizes, any GQA group.  The plain causal softmax
// kernels for d = 128 are in attention.hip, values that are part of the keys in
// attention_latent.hip.
//
// Layouts: q [T, Hq, DK], k cache [num_blocks, Hkv, 64, DK], v cache
// [num_blocks, Hkv, 64, DV], out [T, Hq, DV].
//
// Three forms:
//   tile   4-wave work items (prompt portions): the item's tokens x G heads are
//          rows, 16 per wave; K / V tiles of one 64-key block go through LDS
//          (LDS-DMA) and are shared by the waves;
//   split  1-wave work items (decode): one 16-row tile, the keys shared out over
//          the 4 waves of a block and over gridDim.z blocks, K straight into MFMA
//          registers, V through a per-wave LDS buffer; merged in LDS, then (z > 1)
//          by attn_split_merge;
//   row    one wave per (token, head), fp32: the 32-bit mode, odd head sizes.
// Both MFMA forms compute S^T = K Q^T (v_mfma_f32_16x16x32_bf16; a lane owns one
// query row), then O^T += V^T P^T with P^T straight from the S^T accumulators and
// V^T from transposed LDS reads, as attention.hip does.
//
// Softmax.  The sink is a key of fixed score without a value: a running sum that
// starts at m = its score, l = 1.  A soft cap bounds every score by +-cap, so while
// e^cap is far inside fp32 (cap <= NOMAX_CAP) the weights e^s need no running
// maximum at all: no row reductions and no rescaling inside the key loop, and
// partial sums over keys (waves, splits) simply add.
#include "attention_masked.h"

namespace {

// ---- row form: one wave per (token, query head).  Lanes take keys for the
// scores and value columns for the sum; everything is fp32.  The 32-bit mode
// runs on it, and head sizes the MFMA forms do not cover.
constexpr int ROW_MAX_DV = 1024;

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
  const int first = first_key(a, qpos);
  const int* bt = a.block_table + (size_t)s * a.max_blocks;
  const float slope = a.slopes ? a.slopes[head] : 0.f;
  const T* vc = a.vc ? (const T*)a.vc : (const T*)a.kc;   // (values inside the keys)
  const int ldv = a.vc ? a.DV : a.DK;
  float m_run = !a.sink ? -INFINITY : a.sinks ? a.sinks[head] : 0.f, l = a.sink ? 1.f : 0.f;
  float o[ROW_MAX_DV / 64];
#pragma unroll
  for (int i = 0; i < ROW_MAX_DV / 64; ++i) o[i] = 0.f;
  const TileWalk walk(a, first, qpos);
  for (int i = 0; i < walk.n; ++i) {
    const int kt = walk.tile(i);
    const size_t blk = (size_t)bt[kt] * a.Hkv + kvh;
    const T* kr = (const T*)a.kc + (blk * KT + lane) * a.DK;
    const int key = kt * KT + lane;
    const bool on = key <= qpos && (key >= first || key < a.keep);
    float sc = 0.f;
    if (on) {
      for (int d = 0; d < a.DK; ++d) sc = fmaf(qs[d], (float)kr[d], sc);
      sc *= a.scale;
      if (a.cap > 0.f) sc = a.cap * tanhf(sc / a.cap);
      sc -= slope * (float)(qpos - key);
    }
    const float mt = wave_max(on ? sc : -INFINITY);     // (every tile of the walk has a visible key)
    const float m_new = fmaxf(m_run, mt);
    const float alpha = expf(m_run - m_new);
    const float p = on ? expf(sc - m_new) : 0.f;
    m_run = m_new;
    l = l * alpha + wave_sum(p);
    __syncthreads();
    ps[lane] = p;
    __syncthreads();
    const int k0 = kt * KT < a.keep ? 0 : max(first - kt * KT, 0), k1 = min(qpos - kt * KT, KT - 1);
#pragma unroll
    for (int i = 0; i < ROW_MAX_DV / 64; ++i) {
      const int d = i * 64 + lane;
      if (d < a.DV) {
        float acc = o[i] * alpha;
        const T* vr = vc + blk * KT * ldv + d;
        for (int k = k0; k <= k1; ++k) acc = fmaf(ps[k], (float)vr[(size_t)k * ldv], acc);
        o[i] = acc;
      }
    }
  }
  const float inv = head_gate<T>(a, t, head) / l;
  T* op = (T*)a.out + ((size_t)t * a.Hq + head) * a.DV;
#pragma unroll
  for (int i = 0; i < ROW_MAX_DV / 64; ++i) {
    const int d = i * 64 + lane;
    if (d < a.DV) op[d] = (T)(o[i] * inv);
  }
}


// ------------------------------------------------------------------ tile form
// blockIdx.x = work item, blockIdx.y = key head x 64-row group of the item
template <int DK, int DV, int MODE>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DK + DV <= 256 ? 3 : 1)))
void attn_tile_kernel(const MaskedAttnArgs a) {
  __shared__ __attribute__((aligned(16))) bf16 smem[KT * (DK + DV)];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int fr = lane & 15, fq = lane >> 4;
  const int Hkv = a.Hkv, G = a.Hq / Hkv;
  const int kvh = blockIdx.y % Hkv, rg = blockIdx.y / Hkv;
  const int s = a.work_seq[blockIdx.x], q0 = a.work_q0[blockIdx.x];
  const int ql = a.q_len[s], cl = a.ctx_len[s], qs = a.q_start[s];
  const int ntok = min(a.item_tokens, ql - q0);         // the item's tokens (<= 0: padding)
  const int row0 = rg * 64;
  if (row0 >= ntok * G) return;                          // whole block, before any barrier
  const int rows = min(ntok * G - row0, 64);
  const int row = wave * 16 + fr;
  const bool valid = row < rows;
  const int rr = row0 + (valid ? row : 0);
  const int tok = q0 + rr / G, head = kvh * G + rr % G;
  const int base = cl - ql;                              // position of the span's first token
  const int qpos = base + tok;
  const int first = first_key(a, qpos);          // first key of this lane's row
  // key tiles of the block, and of this wave's rows
  const int b_lo = first_key(a, base + q0 + row0 / G), b_hi = base + q0 + (row0 + rows - 1) / G;
  const int w0 = min(row0 + wave * 16, row0 + rows - 1), w1 = min(row0 + wave * 16 + 15, row0 + rows - 1);
  const int wp0 = base + q0 + w0 / G, wp1 = base + q0 + w1 / G;   // the wave's positions
  const int w_lo = first_key(a, wp0), w_in = first_key(a, wp1);
  const bool w_on = wave * 16 < rows;

  bf16x8 qf[DK / 32];
  {
    const bf16* qp = (const bf16*)a.q + ((size_t)(qs + tok) * a.Hq + head) * DK + 8 * fq;
#pragma unroll
    for (int ks = 0; ks < DK / 32; ++ks) qf[ks] = *reinterpret_cast<const bf16x8*>(qp + 32 * ks);
  }
  const ScoreConst kc = score_const<MODE>(a, head);
  Run st = run_start<MODE>(a, head, a.sink, fq);
  f32x4 o[DV / 16];
#pragma unroll
  for (int i = 0; i < DV / 16; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};

  bf16* Kl = smem;
  bf16* Vl = smem + KT * DK;
  const KeyFrag<DK> kfrag(Kl, fr, fq);
  const TileWalk walk(a, b_lo, b_hi);
  const int* bt = a.block_table + (size_t)s * a.max_blocks;
  int bt_v = 0;                                          // 64 table entries per load
  for (int i = 0; i < walk.n; ++i) {
    if ((i & 63) == 0) bt_v = i + lane < walk.n ? bt[walk.tile(i + lane)] : 0;
    const int kt = walk.tile(i);
    const size_t blk = (size_t)__builtin_amdgcn_readlane(bt_v, i & 63) * Hkv + kvh;
    stage_rows<DK, 0, DK / 32>((const bf16*)a.kc + blk * (KT * DK), Kl, wave * (DK / 32), lane);
    stage_rows<DV, 0, DV / 32>((const bf16*)a.vc + blk * (KT * DV), Vl, wave * (DV / 32), lane);
    __syncthreads();                                     // drains the LDS-DMA
    if (b_hi - kt * KT < KT - 1) {                       // rows past the last key: zero their values
      const int r0 = b_hi - kt * KT + 1;
      for (int c = r0 * (DV / 8) + threadIdx.x; c < KT * (DV / 8); c += 256)
        *reinterpret_cast<u32x4*>(Vl + c * 8) = u32x4{0, 0, 0, 0};
      __syncthreads();
    }
    const int k_lo = kt * KT, k_hi = k_lo + KT - 1;
    if (w_on && k_lo <= wp1 && (k_hi >= w_lo || k_lo < a.keep)) {   // (wave-uniform) some row of the wave sees it
      f32x4 sacc[4];
#pragma unroll
      for (int nt = 0; nt < 4; ++nt) {
        sacc[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < DK / 32; ++ks) sacc[nt] = mfma16x16x32(kfrag.at(nt * 16, ks), qf[ks], sacc[nt]);
      }
      bf16x8 pf[2];
      const int lo = first - k_lo, hi = qpos - k_lo, keep = a.keep - k_lo;
      const float alpha = (k_hi <= wp0 && (k_lo >= w_in || keep >= KT))
                              ? tile_weights<MODE, false>(sacc, pf, st, kc, lo, hi, keep, fq)
                              : tile_weights<MODE, true>(sacc, pf, st, kc, lo, hi, keep, fq);
      if constexpr (MODE != CAPPED_NOMAX) {
#pragma unroll
        for (int dt = 0; dt < DV / 16; ++dt) o[dt] *= alpha;
      }
      tile_pv<DV>(Vl, pf, o, lane);
    }
    __syncthreads();
  }
  float l = st.l + __shfl_xor(st.l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (!valid) return;
  const float inv = l > 0.f ? head_gate<bf16>(a, qs + tok, head) / l : 0.f;
  bf16* op = (bf16*)a.out + ((size_t)(qs + tok) * a.Hq + head) * DV + 4 * fq;
#pragma unroll
  for (int dt = 0; dt < DV / 16; ++dt) {
    bf16x4 w;
#pragma unroll
    for (int r = 0; r < 4; ++r) w[r] = (bf16)(o[dt][r] * inv);
    *reinterpret_cast<bf16x4*>(op + dt * 16) = w;
  }
}

// ----------------------------------------------------------------- split form
// blockIdx.x = work item, .y = key head x 16-row group, .z = key split.  Wave w
// of split z takes every (4 nz)-th tile of the item, from 4 z + w on.
template <int DK, int DV, int MODE>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DK + DV <= 256 ? 2 : 1)))
void attn_split_kernel(const MaskedAttnArgs a) {
  constexpr int NWV = 4;
  __shared__ __attribute__((aligned(16))) bf16 smem[NWV * KT * DV];   // V tiles, then the waves' O
  __shared__ float red_m[NWV][16], red_l[NWV][16];
  __shared__ int s_last;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int fr = lane & 15, fq = lane >> 4;
  const int Hkv = a.Hkv, G = a.Hq / Hkv;
  const int kvh = blockIdx.y % Hkv, rg = blockIdx.y / Hkv;
  const int z = blockIdx.z, nz = gridDim.z;
  const int s = a.work_seq[blockIdx.x], q0 = a.work_q0[blockIdx.x];
  const int ql = a.q_len[s], cl = a.ctx_len[s], qs = a.q_start[s];
  const int ntok = min(a.item_tokens, ql - q0);
  const int row0 = rg * 16;
  if (row0 >= ntok * G) return;                          // whole block, before any barrier
  const int rows = min(ntok * G - row0, 16);
  const bool valid = fr < rows;
  const int rr = row0 + (valid ? fr : 0);
  const int tok = q0 + rr / G, head = kvh * G + rr % G;
  const int base = cl - ql, qpos = base + tok;
  const int first = first_key(a, qpos);
  const int p0 = base + q0 + row0 / G, p1 = base + q0 + (row0 + rows - 1) / G;
  const int lo = first_key(a, p0), in = first_key(a, p1);

  bf16x8 qf[DK / 32];
  {
    const bf16* qp = (const bf16*)a.q + ((size_t)(qs + tok) * a.Hq + head) * DK + 8 * fq;
#pragma unroll
    for (int ks = 0; ks < DK / 32; ++ks) qf[ks] = *reinterpret_cast<const bf16x8*>(qp + 32 * ks);
  }
  const ScoreConst kc = score_const<MODE>(a, head);
  Run st = run_start<MODE>(a, head, a.sink && z == 0 && wave == 0, fq);
  f32x4 o[DV / 16];
#pragma unroll
  for (int i = 0; i < DV / 16; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};

  bf16* Vl = smem + wave * (KT * DV);
  const TileWalk walk(a, lo, p1);
  const int step = NWV * nz;
  const int* bt = a.block_table + (size_t)s * a.max_blocks;
  int left = 0, bt_v = 0;
  for (int it = z * NWV + wave; it < walk.n; it += step, --left) {
    if (left == 0) {                                     // the wave's next 64 table entries
      const int i = it + lane * step;
      bt_v = i < walk.n ? bt[walk.tile(i)] : 0;
      left = 64;
    }
    const int kt = walk.tile(it);
    const size_t blk = (size_t)__builtin_amdgcn_readlane(bt_v, 64 - left) * Hkv + kvh;
    const bf16* kp = (const bf16*)a.kc + blk * (KT * DK) + fr * DK + 8 * fq;
    bf16x8 kf[4][DK / 32];
#pragma unroll
    for (int nt = 0; nt < 4; ++nt)
#pragma unroll
      for (int ks = 0; ks < DK / 32; ++ks)
        kf[nt][ks] = *reinterpret_cast<const bf16x8*>(kp + nt * 16 * DK + 32 * ks);
    stage_rows<DV, 0, DV / 8>((const bf16*)a.vc + blk * (KT * DV), Vl, 0, lane);
    f32x4 sacc[4];
#pragma unroll
    for (int nt = 0; nt < 4; ++nt) {
      sacc[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < DK / 32; ++ks) sacc[nt] = mfma16x16x32(kf[nt][ks], qf[ks], sacc[nt]);
    }
    const int k_lo = kt * KT, k_hi = k_lo + KT - 1;
    bf16x8 pf[2];
    const int wlo = first - k_lo, whi = qpos - k_lo, keep = a.keep - k_lo;
    const float alpha = (k_hi <= p0 && (k_lo >= in || keep >= KT))
                            ? tile_weights<MODE, false>(sacc, pf, st, kc, wlo, whi, keep, fq)
                            : tile_weights<MODE, true>(sacc, pf, st, kc, wlo, whi, keep, fq);
    if constexpr (MODE != CAPPED_NOMAX) {
#pragma unroll
      for (int dt = 0; dt < DV / 16; ++dt) o[dt] *= alpha;
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");     // the wave's V tile is in LDS
    if (p1 - k_lo < KT - 1) {                            // rows past the last key: zero their values
      for (int c = (p1 - k_lo + 1) * (DV / 8) + lane; c < KT * (DV / 8); c += 64)
        *reinterpret_cast<u32x4*>(Vl + c * 8) = u32x4{0, 0, 0, 0};
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    }
    tile_pv<DV>(Vl, pf, o, lane);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // V is read before the next DMA lands
  }

  // ---- merge the waves: O [16][DV] fp32 per wave in its own V buffer
  float l = st.l + __shfl_xor(st.l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (fq == 0) {
    red_m[wave][fr] = st.m;
    red_l[wave][fr] = l;
  }
  float* Ow = reinterpret_cast<float*>(Vl);
#pragma unroll
  for (int dt = 0; dt < DV / 16; ++dt)
    *reinterpret_cast<f32x4*>(Ow + fr * DV + dt * 16 + 4 * fq) = o[dt];
  __syncthreads();
  const int r = threadIdx.x >> 4, c0 = (threadIdx.x & 15) * 4;
  const bool live = r < rows;
  float m = red_m[0][r], wgt[NWV], lt = 0.f;
#pragma unroll
  for (int w = 1; w < NWV; ++w) m = fmaxf(m, red_m[w][r]);
  const float mu = m == -INFINITY ? 0.f : m;
#pragma unroll
  for (int w = 0; w < NWV; ++w) {
    wgt[w] = MODE == CAPPED_NOMAX ? 1.f : fexp2(red_m[w][r] - mu);
    lt += wgt[w] * red_l[w][r];
  }
  const int r2 = row0 + (live ? r : 0);
  const size_t orow = (size_t)(qs + q0 + r2 / G) * a.Hq + kvh * G + r2 % G;
  f32x4 v[DV / 64];
#pragma unroll
  for (int i = 0; i < DV / 64; ++i) {
    v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < NWV; ++w)
      v[i] += *reinterpret_cast<const f32x4*>(reinterpret_cast<const float*>(smem + w * (KT * DV)) + r * DV +
                                              c0 + 64 * i) * wgt[w];
  }
  bf16* op = (bf16*)a.out + orow * DV + c0;
  const float gate = head_gate<bf16>(a, orow / a.Hq, (int)(orow % a.Hq));
  auto put = [&](float inv) {
    inv *= gate;
#pragma unroll
    for (int i = 0; i < DV / 64; ++i) {
      bf16x4 b;
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = (bf16)(v[i][j] * inv);
      *reinterpret_cast<bf16x4*>(op + 64 * i) = b;
    }
  };
  if (nz == 1) {
    if (live) put(lt > 0.f ? 1.f / lt : 0.f);
    return;
  }
  // ---- merge the splits: every block stores its unnormalised O and (m, l)
  // write-through (sc1), drains them and takes the item's ticket; the last one
  // adds all partials up, read back in split order (sc1), so the result does not
  // depend on the order of arrival.  Every wave reaches both barriers.
  const auto rso = __builtin_amdgcn_make_buffer_rsrc(a.split_o, (short)0, 0x7FFFFFFF, 0x00020000);
  const auto rsm = __builtin_amdgcn_make_buffer_rsrc(a.split_ml, (short)0, 0x7FFFFFFF, 0x00020000);
  if (live) {
#pragma unroll
    for (int i = 0; i < DV / 64; ++i)
      __builtin_amdgcn_raw_buffer_store_b128(__builtin_bit_cast(u32x4, v[i]), rso,
                                             (unsigned)((((size_t)z * a.rows + orow) * DV + c0 + 64 * i) * 4), 0, 16);
    if ((threadIdx.x & 15) == 0)
      __builtin_amdgcn_raw_buffer_store_b64(u32x2{__builtin_bit_cast(unsigned, m), __builtin_bit_cast(unsigned, lt)},
                                            rsm, (unsigned)(((size_t)z * a.rows + orow) * 8), 0, 16);
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (threadIdx.x == 0) {
    int* cnt = a.tickets + (size_t)blockIdx.x * gridDim.y + blockIdx.y;
    const int old = __hip_atomic_fetch_add(cnt, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    if (old == nz - 1) __hip_atomic_store(cnt, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    s_last = old == nz - 1;
  }
  __syncthreads();
  if (!s_last || !live) return;
  auto ml = [&](int j) {
    return __builtin_amdgcn_raw_buffer_load_b64(rsm, (unsigned)(((size_t)j * a.rows + orow) * 8), 0, 16);
  };
  float mx = 0.f;
  if constexpr (MODE != CAPPED_NOMAX) {
    mx = -INFINITY;
#pragma unroll 8
    for (int j = 0; j < nz; ++j) mx = fmaxf(mx, __builtin_bit_cast(float, (unsigned)ml(j)[0]));
    mx = mx == -INFINITY ? 0.f : mx;
  }
  lt = 0.f;
#pragma unroll
  for (int i = 0; i < DV / 64; ++i) v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int j = 0; j < nz; ++j) {
    const auto p = ml(j);
    const float w = MODE == CAPPED_NOMAX ? 1.f : fexp2(__builtin_bit_cast(float, (unsigned)p[0]) - mx);
    lt += w * __builtin_bit_cast(float, (unsigned)p[1]);
#pragma unroll
    for (int i = 0; i < DV / 64; ++i)
      v[i] += __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(
                  rso, (unsigned)((((size_t)j * a.rows + orow) * DV + c0 + 64 * i) * 4), 0, 16)) * w;
  }
  put(lt > 0.f ? 1.f / lt : 0.f);
}

template <int DK, int DV, int MODE>
void launch_mode(const MaskedAttnArgs& a, int nwork, int form, int nz, hipStream_t s) {
  const int G = a.Hq / a.Hkv;
  if (form == 4) {
    const int groups = (a.item_tokens * G + 63) / 64;
    attn_tile_kernel<DK, DV, MODE><<<dim3(nwork, a.Hkv * groups), 256, 0, s>>>(a);
    return;
  }
  const int groups = (a.item_tokens * G + 15) / 16;
  attn_split_kernel<DK, DV, MODE><<<dim3(nwork, a.Hkv * groups, nz), 256, 0, s>>>(a);
}

template <int DK, int DV>
void launch_dims(const MaskedAttnArgs& a, int nwork, int form, int nz, hipStream_t s) {
  if (a.slopes) launch_mode<DK, DV, BIASED>(a, nwork, form, nz, s);
  else if (a.cap <= 0.f) launch_mode<DK, DV, PLAIN>(a, nwork, form, nz, s);
  else if (a.cap <= NOMAX_CAP) launch_mode<DK, DV, CAPPED_NOMAX>(a, nwork, form, nz, s);
  else launch_mode<DK, DV, CAPPED>(a, nwork, form, nz, s);
}

template <int DK>
int launch_dk(const MaskedAttnArgs& a, int nwork, int form, int nz, hipStream_t s) {
  switch (a.DV) {
    case 64: launch_dims<DK, 64>(a, nwork, form, nz, s); return 0;
    case 128: launch_dims<DK, 128>(a, nwork, form, nz, s); return 0;
    case 192: launch_dims<DK, 192>(a, nwork, form, nz, s); return 0;
    case 256: launch_dims<DK, 256>(a, nwork, form, nz, s); return 0;
    default: return 3;
  }
}

}  // namespace

// One work list (form 4: the 4-wave items, 1: the 1-wave items, whose keys go
// over nz splits); nonzero: head sizes outside 64 / 128 / 192 / 256
int launch_attn_masked(const MaskedAttnArgs& args, int nwork, int form, int nz, hipStream_t s) {
  MaskedAttnArgs a = args;
  if (nwork <= 0) return 0;
  if ((form != 1 && form != 4) || (a.slopes && a.cap > 0.f)) return 1;
  if (nz < 1 || (form == 4 && nz != 1) || (nz > 1 && (!a.split_o || !a.split_ml))) return 2;
  if (nz > 1) {
    // tickets: one per item, key head and row group (the split-KV tickets of attention.hip)
    const long long groups = (a.item_tokens * (a.Hq / a.Hkv) + 15) / 16;
    a.tickets = attn_split_counters();
    if (!a.tickets || nwork * a.Hkv * groups > ATTN_SPLIT_TICKETS ||
        (long long)nz * a.rows * a.DV * 4 >= (1ll << 31))
      nz = 1;                                            // one block per item walks all its keys
  }
  switch (a.DK) {
    case 64: return launch_dk<64>(a, nwork, form, nz, s);
    case 128: return launch_dk<128>(a, nwork, form, nz, s);
    case 192: return launch_dk<192>(a, nwork, form, nz, s);
    case 256: return launch_dk<256>(a, nwork, form, nz, s);
    default: return 3;
  }
}

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
