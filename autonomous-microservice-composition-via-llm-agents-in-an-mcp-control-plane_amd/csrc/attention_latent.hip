// Latent attention over the paged cache: one key head for every query head, and
// the values are the first DV columns of the cached row.  Masks, sink and gate as
// in attention_masked.hip.
//
// Layouts: q [T, Hq, DK] (absorbed queries), cache [num_blocks, 1, 64, DK],
// out [T, Hq, DV].
//
// blockIdx.x = work item, .y = 64-row group (the item's tokens x Hq heads), .z =
// key split.  Each of the 4 waves owns 16 rows; one 64-key tile of whole rows goes
// through LDS (LDS-DMA) and serves K Q^T and P V both, so HBM and L2 give every
// cached byte once per row group.  Split keys are merged by the last block of a
// row group, in split order.
#include "attention_masked.h"

namespace {

template <int DK, int DV>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DK > 320 ? 1 : 2)))
void attn_latent_kernel(const MaskedAttnArgs a) {
  constexpr int MODE = PLAIN;
  __shared__ __attribute__((aligned(16))) bf16 Kl[KT * DK];
  __shared__ int s_last;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int fr = lane & 15, fq = lane >> 4;
  const int G = a.Hq, z = blockIdx.z, nz = gridDim.z;
  const int s = a.work_seq[blockIdx.x], q0 = a.work_q0[blockIdx.x];
  const int ql = a.q_len[s], cl = a.ctx_len[s], qs = a.q_start[s];
  const int ntok = min(a.item_tokens, ql - q0);          // the item's tokens (<= 0: padding)
  const int row0 = blockIdx.y * 64;
  if (row0 >= ntok * G) return;                          // whole block, before any barrier
  const int rows = min(ntok * G - row0, 64);
  const int row = wave * 16 + fr;
  const bool valid = row < rows;
  const int rr = row0 + (valid ? row : 0);
  const int tok = q0 + rr / G, head = rr % G;
  const int base = cl - ql;                              // position of the span's first token
  const int qpos = base + tok, first = first_key(a, qpos);
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
  Run st = run_start<MODE>(a, head, a.sink && z == 0, fq);
  f32x4 o[DV / 16];
#pragma unroll
  for (int i = 0; i < DV / 16; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};

  const TileWalk walk(a, b_lo, b_hi);
  const int* bt = a.block_table + (size_t)s * a.max_blocks;
  int left = 0, bt_v = 0;
  for (int it = z; it < walk.n; it += nz, --left) {
    if (left == 0) {                                     // the next 64 table entries
      const int i = it + lane * nz;
      bt_v = i < walk.n ? bt[walk.tile(i)] : 0;
      left = 64;
    }
    const int kt = walk.tile(it);
    const size_t blk = (size_t)__builtin_amdgcn_readlane(bt_v, 64 - left);
    stage_rows<DK, 0, DK / 32>((const bf16*)a.kc + blk * (KT * DK), Kl, wave * (DK / 32), lane);
    __syncthreads();                                     // drains the LDS-DMA
    const int k_lo = kt * KT, k_hi = k_lo + KT - 1;
    if (b_hi < k_hi) {                                   // rows past the last key: zero them
      for (int c = (b_hi - k_lo + 1) * (DK / 8) + threadIdx.x; c < KT * (DK / 8); c += 256)
        *reinterpret_cast<u32x4*>(Kl + c * 8) = u32x4{0, 0, 0, 0};
      __syncthreads();
    }
    if (w_on && k_lo <= wp1 && (k_hi >= w_lo || k_lo < a.keep)) {   // (wave-uniform) some row of the wave sees it
      f32x4 sacc[4];
#pragma unroll
      for (int nt = 0; nt < 4; ++nt) {
        sacc[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int kr = nt * 16 + fr;
#pragma unroll
        for (int ks = 0; ks < DK / 32; ++ks) {
          const bf16x8 kf = *reinterpret_cast<const bf16x8*>(Kl + kr * DK + (((ks * 4 + fq) ^ (kr & 7)) << 3));
          sacc[nt] = mfma16x16x32(kf, qf[ks], sacc[nt]);
        }
      }
      bf16x8 pf[2];
      const int lo = first - k_lo, hi = qpos - k_lo, keep = a.keep - k_lo;
      const float alpha = (k_hi <= wp0 && (k_lo >= w_in || keep >= KT))
                              ? tile_weights<MODE, false>(sacc, pf, st, kc, lo, hi, keep, fq)
                              : tile_weights<MODE, true>(sacc, pf, st, kc, lo, hi, keep, fq);
#pragma unroll
      for (int dt = 0; dt < DV / 16; ++dt) o[dt] *= alpha;
      tile_pv<DV, DK>(Kl, pf, o, lane);
    }
    __syncthreads();
  }
  float l = st.l + __shfl_xor(st.l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  const size_t orow = (size_t)(qs + tok) * a.Hq + head;
  const float gate = head_gate<bf16>(a, qs + tok, head);
  bf16* op = (bf16*)a.out + orow * DV + 4 * fq;
  auto put = [&](float inv) {
    inv *= gate;
#pragma unroll
    for (int dt = 0; dt < DV / 16; ++dt) {
      bf16x4 w;
#pragma unroll
      for (int r = 0; r < 4; ++r) w[r] = (bf16)(o[dt][r] * inv);
      *reinterpret_cast<bf16x4*>(op + dt * 16) = w;
    }
  };
  if (nz == 1) {
    if (valid) put(l > 0.f ? 1.f / l : 0.f);
    return;
  }
  // ---- merge the splits, as attn_split_kernel does: unnormalised O and (m, l)
  // go out write-through (sc1) and are drained before the ticket; the last block
  // reads them back in split order.  Every wave reaches both barriers.
  const auto rso = __builtin_amdgcn_make_buffer_rsrc(a.split_o, (short)0, 0x7FFFFFFF, 0x00020000);
  const auto rsm = __builtin_amdgcn_make_buffer_rsrc(a.split_ml, (short)0, 0x7FFFFFFF, 0x00020000);
  auto part = [&](int j, int dt) { return (unsigned)((((size_t)j * a.rows + orow) * DV + dt * 16 + 4 * fq) * 4); };
  if (valid) {
#pragma unroll
    for (int dt = 0; dt < DV / 16; ++dt)
      __builtin_amdgcn_raw_buffer_store_b128(__builtin_bit_cast(u32x4, o[dt]), rso, part(z, dt), 0, 16);
    if (fq == 0)
      __builtin_amdgcn_raw_buffer_store_b64(
          u32x2{__builtin_bit_cast(unsigned, st.m), __builtin_bit_cast(unsigned, l)}, rsm,
          (unsigned)(((size_t)z * a.rows + orow) * 8), 0, 16);
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
  if (!s_last || !valid) return;
  auto ml = [&](int j) {
    return __builtin_amdgcn_raw_buffer_load_b64(rsm, (unsigned)(((size_t)j * a.rows + orow) * 8), 0, 16);
  };
  float mx = -INFINITY;
#pragma unroll 8
  for (int j = 0; j < nz; ++j) mx = fmaxf(mx, __builtin_bit_cast(float, (unsigned)ml(j)[0]));
  mx = mx == -INFINITY ? 0.f : mx;
  l = 0.f;
#pragma unroll
  for (int dt = 0; dt < DV / 16; ++dt) o[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int j = 0; j < nz; ++j) {
    const auto p = ml(j);
    const float w = fexp2(__builtin_bit_cast(float, (unsigned)p[0]) - mx);
    l += w * __builtin_bit_cast(float, (unsigned)p[1]);
#pragma unroll
    for (int dt = 0; dt < DV / 16; ++dt)
      o[dt] += __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(rso, part(j, dt), 0, 16)) * w;
  }
  put(l > 0.f ? 1.f / l : 0.f);
}

template <int DK, int DV>
int launch_pair(const MaskedAttnArgs& a, int nwork, int nz, hipStream_t s) {
  const int groups = (a.item_tokens * a.Hq + 63) / 64;
  attn_latent_kernel<DK, DV><<<dim3(nwork, groups, nz), 256, 0, s>>>(a);
  return 0;
}

}  // namespace

// One work list; 3: a (DK, DV) pair without a kernel (the row form takes it)
int launch_attn_latent(const MaskedAttnArgs& args, int nwork, int nz, hipStream_t s) {
  MaskedAttnArgs a = args;
  if (nwork <= 0) return 0;
  if (a.Hkv != 1 || a.cap > 0.f || a.slopes) return 1;
  if (nz < 1 || (nz > 1 && (!a.split_o || !a.split_ml))) return 2;
  if (nz > 1) {
    const long long groups = (a.item_tokens * a.Hq + 63) / 64;
    a.tickets = attn_split_counters();
    if (!a.tickets || nwork * groups > ATTN_SPLIT_TICKETS || (long long)nz * a.rows * a.DV * 4 >= (1ll << 31))
      nz = 1;                                            // one block per item walks all its keys
  }
  switch (a.DK * 1024 + a.DV) {
    case 64 * 1024 + 64: return launch_pair<64, 64>(a, nwork, nz, s);
    case 128 * 1024 + 64: return launch_pair<128, 64>(a, nwork, nz, s);
    case 128 * 1024 + 128: return launch_pair<128, 128>(a, nwork, nz, s);
    case 192 * 1024 + 128: return launch_pair<192, 128>(a, nwork, nz, s);
    case 192 * 1024 + 192: return launch_pair<192, 192>(a, nwork, nz, s);
    case 256 * 1024 + 192: return launch_pair<256, 192>(a, nwork, nz, s);
    case 256 * 1024 + 256: return launch_pair<256, 256>(a, nwork, nz, s);
    case 320 * 1024 + 256: return launch_pair<320, 256>(a, nwork, nz, s);
    case 448 * 1024 + 384: return launch_pair<448, 384>(a, nwork, nz, s);
    case 576 * 1024 + 512: return launch_pair<576, 512>(a, nwork, nz, s);
    default: return 3;
  }
}
