// Latent attention over the paged cache: one row [latent | rotated key] per token
// is what every head's key and value come from.  Masks, sink and gate as in
// attention_masked.hip.
//
//   absorbed   (decode, short portions)  q [T, Hq, DK] already holds the queries
//              taken through the key projection; the cached row is the one key
//              head, its first DV columns the values; out [T, Hq, DV] latents.
//   expanded   (long portions)  keys and values of every head have been projected
//              from the cached rows once; plain attention per head on them, at
//              dim + rot and value size instead of twice the latent's.
//
// Both compute S^T = K Q^T and O^T += V^T P^T as attention_masked.hip does.
#include "attention_masked.h"
#include "rows.h"

namespace {

// ------------------------------------------------------------------- absorbed
// blockIdx.x = work item, .y = group of 16 R rows (the item's tokens x Hq heads; a
// block takes every gridDim.y-th), .z = key split.  One 64-key tile of whole rows goes through LDS and serves K and
// V both.  The 4 R waves share the rows: wave 4 t + w scores keys [16 w, 16 w + 16)
// of the tile for row tile t, the weights meet in LDS, then every wave sums its own
// 16-column tiles of the values for all rows - so the staged values are read from
// LDS once for all R row tiles, and no wave is idle when there are few rows.
template <int DK, int DV, int R>
__global__ __launch_bounds__(256 * R) __attribute__((amdgpu_waves_per_eu(2)))
void attn_latent_kernel(const MaskedAttnArgs a) {
  constexpr int NW = 4 * R, NR = 16 * R, PLD = KT + 8;
  constexpr int CT = DV / 16, ND = (CT + NW - 1) / NW;     // column tiles: all, per wave
  constexpr int DMA = DK / 8 / NW;                         // LDS-DMA instructions per wave and tile
  constexpr int VM_DMA = 0x0F70 | (DMA & 15) | (DMA >> 4) << 14;   // s_waitcnt vmcnt(DMA)
  // two tile buffers as two objects: the next tile's DMA does not alias this one's reads
  __shared__ __attribute__((aligned(16))) bf16 K0[KT * DK], K1[KT * DK];
  __shared__ __attribute__((aligned(16))) bf16 Pl[NR * PLD];
  __shared__ float red[4][NR];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int fr = lane & 15, fq = lane >> 4, kw = wave & 3, own = wave >> 2;
  const int G = a.Hq, z = blockIdx.z, nz = gridDim.z;
  const int s = a.work_seq[blockIdx.x], q0 = a.work_q0[blockIdx.x];
  const int ql = a.q_len[s], cl = a.ctx_len[s], qs = a.q_start[s];
  const int ntok = min(a.item_tokens, ql - q0);          // the item's tokens (<= 0: padding)
  if (a.skip_q > 0 && ql >= a.skip_q) return;            // whole block, before any barrier
  for (int row0 = blockIdx.y * NR; row0 < ntok * G; row0 += gridDim.y * NR) {
    const int rows = min(ntok * G - row0, NR);
    const int base = cl - ql;                              // position of the span's first token
    float m[R], l_own;
#pragma unroll
    for (int t = 0; t < R; ++t) {
      const Run st = run_start<PLAIN>(a, (row0 + min(t * 16 + fr, rows - 1)) % G, a.sink && z == 0, fq);
      m[t] = st.m;
      if (t == own) l_own = kw ? 0.f : st.l;               // (the waves' sums add)
    }
    const int rr = row0 + min(own * 16 + fr, rows - 1);
    const int qpos = base + q0 + rr / G, first = first_key(a, qpos);
    bf16x8 qf[DK / 32];
    {
      const bf16* qp = (const bf16*)a.q + ((size_t)(qs + q0 + rr / G) * a.Hq + rr % G) * DK + 8 * fq;
#pragma unroll
      for (int ks = 0; ks < DK / 32; ++ks) qf[ks] = *reinterpret_cast<const bf16x8*>(qp + 32 * ks);
    }
    const int b_lo = first_key(a, base + q0 + row0 / G), b_hi = base + q0 + (row0 + rows - 1) / G;
    const float ka = a.scale * LOG2E;
    f32x4 o[R][ND];
#pragma unroll
    for (int t = 0; t < R; ++t)
#pragma unroll
      for (int i = 0; i < ND; ++i) o[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};
    const TileWalk walk(a, b_lo, b_hi);
    const int* bt = a.block_table + (size_t)s * a.max_blocks;
    // the block's tiles are z, z + nz, ...; table entries come 64 at a time
    int bt_at = -1, bt_v = 0;
    auto stage = [&](int i, bf16* dst) {                   // tile i of the block's
      if (i >> 6 != bt_at) {
        bt_at = i >> 6;
        const int e = z + ((i & ~63) + lane) * nz;
        bt_v = e < walk.n ? bt[walk.tile(e)] : 0;
        __builtin_amdgcn_s_waitcnt(0x0F70);                // vmcnt(0), here and not at every use
      }
      const size_t blk = (size_t)__builtin_amdgcn_readlane(bt_v, i & 63);
      stage_rows<DK, 0, DMA>((const bf16*)a.kc + blk * (KT * DK), dst, wave * DMA, lane);
    };
    // the barriers inside a tile order LDS only: the next tile's DMA stays in flight
    auto lds_barrier = [] { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); };
    const int mine = walk.n > z ? (walk.n - z + nz - 1) / nz : 0;
    auto tile = [&](int i, bf16* Kl) {
      const int k_lo = walk.tile(z + i * nz) * KT;
      if (i + 1 < mine) __builtin_amdgcn_s_waitcnt(VM_DMA);   // this tile's DMA has landed, the next one's may not
      else __builtin_amdgcn_s_waitcnt(0x0F70);
      lds_barrier();
      const KeyFrag<DK> kfrag(Kl, kw * 16 + fr, fq);
      const ValFrag<DK, 1> vfrag(Kl, lane, wave);          // (NW % 4 == 0: one base serves all its tiles)
      if (b_hi - k_lo < KT - 1) {                          // rows past the last key: zero them
        for (int c = (b_hi - k_lo + 1) * (DK / 8) + threadIdx.x; c < KT * (DK / 8); c += NW * 64)
          *reinterpret_cast<u32x4*>(Kl + c * 8) = u32x4{0, 0, 0, 0};
        lds_barrier();
      }
      f32x4 sacc = f32x4{0.f, 0.f, 0.f, 0.f}, sodd = sacc;   // two chains
#pragma unroll
      for (int ks = 0; ks < DK / 32; ks += 2) {
        sacc = mfma16x16x32(kfrag.at(0, ks), qf[ks], sacc);
        sodd = mfma16x16x32(kfrag.at(0, ks + 1), qf[ks + 1], sodd);
      }
      sacc += sodd;
      float mx = -INFINITY;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = k_lo + kw * 16 + fq * 4 + r;
        const bool on = (key <= qpos) & ((key >= first) | (key < a.keep));
        sacc[r] = on ? sacc[r] * ka : -INFINITY;
        mx = fmaxf(mx, sacc[r]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (fq == 0) red[kw][own * 16 + fr] = mx;
      lds_barrier();
      bool scale = false;
      float alpha[R];
#pragma unroll
      for (int t = 0; t < R; ++t) {
        const int i = t * 16 + fr;
        const float m_new = fmaxf(m[t], fmaxf(fmaxf(red[0][i], red[1][i]), fmaxf(red[2][i], red[3][i])));
        const float mu = m_new == -INFINITY ? 0.f : m_new;  // every key masked so far
        alpha[t] = fexp2(m[t] - mu);
        m[t] = m_new;
        scale |= alpha[t] != 1.f;
        if (t == own) {                                    // (wave-uniform)
          bf16x4 p;
          float sum = 0.f;
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float w = fexp2(sacc[r] - mu);
            sum += w;
            p[r] = (bf16)w;
          }
          l_own = l_own * alpha[t] + sum;
          *reinterpret_cast<bf16x4*>(Pl + i * PLD + kw * 16 + fq * 4) = p;
        }
      }
      lds_barrier();
      bf16x8 pf[R][2];                                     // key order of ValFrag: 32 k2 + 4 fq, + 16
#pragma unroll
      for (int t = 0; t < R; ++t)
#pragma unroll
        for (int k2 = 0; k2 < 2; ++k2) {
          const bf16* pp = Pl + (t * 16 + fr) * PLD + k2 * 32 + fq * 4;
          const bf16x4 p0 = *reinterpret_cast<const bf16x4*>(pp), p1 = *reinterpret_cast<const bf16x4*>(pp + 16);
          pf[t][k2] = bf16x8{p0[0], p0[1], p0[2], p0[3], p1[0], p1[1], p1[2], p1[3]};
        }
      if (__any(scale)) {
#pragma unroll
        for (int t = 0; t < R; ++t)
#pragma unroll
          for (int i = 0; i < ND; ++i) o[t][i] *= alpha[t];
      }
#pragma unroll
      for (int i = 0; i < ND; ++i) {
        if (CT % NW && wave + i * NW >= CT) break;         // (wave-uniform)
#pragma unroll
        for (int k2 = 0; k2 < 2; ++k2) {
          const bf16x8 vf = vfrag.at(0, k2, ((wave >> 2) + i * R) * 64);
#pragma unroll
          for (int t = 0; t < R; ++t) o[t][i] = mfma16x16x32(vf, pf[t][k2], o[t][i]);
        }
      }
      lds_barrier();                                       // the buffer is free again
      if (i + 2 < mine) stage(i + 2, Kl);
    };
    if (mine) {
      stage(0, K0);
      __builtin_amdgcn_s_waitcnt(VM_DMA);                  // the queries are here
    }
    if (mine > 1) stage(1, K1);
    for (int i = 0; i < mine; i += 2) {
      tile(i, K0);
      if (i + 1 < mine) tile(i + 1, K1);
    }
    // ---- the waves' sums, then out, or (split keys) the unnormalised partials
    l_own += __shfl_xor(l_own, 16, 64);
    l_own += __shfl_xor(l_own, 32, 64);
    if (fq == 0) red[kw][own * 16 + fr] = l_own;
    __syncthreads();
#pragma unroll
    for (int t = 0; t < R; ++t) {
      const int i = t * 16 + fr;
      if (i >= rows) continue;
      const int ri = row0 + i, head = ri % G, col = wave * 16 + 4 * fq;
      const size_t tok = (size_t)(qs + q0 + ri / G), orow = tok * a.Hq + head;
      const float l = red[0][i] + red[1][i] + red[2][i] + red[3][i];
      if (nz > 1) {
        float* po = a.split_o + ((size_t)z * a.rows + orow) * DV + col;
#pragma unroll
        for (int d = 0; d < ND; ++d)
          if (CT % NW == 0 || wave + d * NW < CT) *reinterpret_cast<f32x4*>(po + d * NW * 16) = o[t][d];
        if (wave == 0 && fq == 0)
          *reinterpret_cast<float2*>(a.split_ml + ((size_t)z * a.rows + orow) * 2) = make_float2(m[t], l);
        continue;
      }
      const float inv = l > 0.f ? head_gate<bf16>(a, tok, head) / l : 0.f;
      bf16* op = (bf16*)a.out + orow * DV + col;
#pragma unroll
      for (int d = 0; d < ND; ++d) {
        if (CT % NW && wave + d * NW >= CT) break;
        bf16x4 w;
#pragma unroll
        for (int r = 0; r < 4; ++r) w[r] = (bf16)(o[t][d][r] * inv);
        *reinterpret_cast<bf16x4*>(op + d * NW * 16) = w;
      }
    }
    lds_barrier();                                         // red and the buffers are free again
  }
}

// merge of split keys, in split order: 128 threads per row of a work item, 4 columns
// each; lane j of a wave holds split j's weight
constexpr int MAX_SPLITS = 64;

__global__ __launch_bounds__(256) void attn_latent_merge_kernel(const MaskedAttnArgs a, int nz) {
  const int lane = threadIdx.x & 63;
  const int s = a.work_seq[blockIdx.x], q0 = a.work_q0[blockIdx.x];
  const int ql = a.q_len[s], rows = min(a.item_tokens, ql - q0) * a.Hq;
  if (a.skip_q > 0 && ql >= a.skip_q) return;
  for (int row = blockIdx.y * 2 + (threadIdx.x >> 7); row < rows; row += gridDim.y * 2) {
    const size_t tok = (size_t)a.q_start[s] + q0 + row / a.Hq, orow = tok * a.Hq + row % a.Hq;
    const float2 ml = lane < nz ? ((const float2*)a.split_ml)[(size_t)lane * a.rows + orow] : make_float2(-INFINITY, 0.f);
    const float mx = wave_max(ml.x), mu = mx == -INFINITY ? 0.f : mx;
    const float wl = fexp2(ml.x - mu), l = wave_sum(wl * ml.y);
    const float inv = l > 0.f ? head_gate<bf16>(a, tok, row % a.Hq) / l : 0.f;
    for (int c = (threadIdx.x & 127) * 4; c < a.DV; c += 512) {
      const float* p = a.split_o + orow * a.DV + c;
      const size_t step = (size_t)a.rows * a.DV;
      f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 16
      for (int j = 0; j < nz; ++j) v += *reinterpret_cast<const f32x4*>(p + j * step) * __shfl(wl, j, 64);
      bf16x4 b;
#pragma unroll
      for (int r = 0; r < 4; ++r) b[r] = (bf16)(v[r] * inv);
      *reinterpret_cast<bf16x4*>((bf16*)a.out + orow * a.DV + c) = b;
    }
  }
}

template <int DK, int DV>
int launch_pair(const MaskedAttnArgs& a, int nwork, int form, int nz, hipStream_t s) {
  // 1-wave items with split keys (decoding): one token's rows in the grid.  Blocks of
  // further tokens would mostly find none, and hold a CU's LDS to see that
  const int rows = (form == 1 && nz > 1 ? 1 : a.item_tokens) * a.Hq;
  if (a.Hq <= 16) attn_latent_kernel<DK, DV, 1><<<dim3(nwork, (rows + 15) / 16, nz), 256, 0, s>>>(a);
  else attn_latent_kernel<DK, DV, 2><<<dim3(nwork, (rows + 31) / 32, nz), 512, 0, s>>>(a);
  if (nz > 1) attn_latent_merge_kernel<<<dim3(nwork, (rows + 1) / 2), 256, 0, s>>>(a, nz);
  return 0;
}

// ------------------------------------------------------------------- expanded
// blockIdx.x = head (heads of one XCD keep to it, with their keys and values in
// its L2), .y = 128-token item.  A wave owns 32 query rows as two MFMA column
// tiles, so that every K and V fragment read from LDS feeds two products.
template <int DK, int DV>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DK + DV <= 320 ? 2 : 1)))
void attn_latent_prefill_kernel(const LatentPrefillArgs a) {
  __shared__ __attribute__((aligned(16))) bf16 smem[KT * (DK + DV)];
  bf16* Kl = smem;
  bf16* Vl = smem + KT * DK;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int fr = lane & 15, fq = lane >> 4;
  const int h = blockIdx.x, s = a.item_seq[blockIdx.y], q0 = a.item_q0[blockIdx.y];
  const int ql = a.q_len[s], base = a.ctx_len[s] - ql, qs = a.q_start[s];
  const int ntok = min(LATENT_ITEM, ql - q0);
  if (ntok <= 0) return;                                 // whole block, before any barrier
  const int b_lo = window_start(a.window, base + q0), b_hi = base + q0 + ntok - 1;
  const bool w_on = wave * 32 < ntok;
  const int wp0 = base + q0 + min(wave * 32, ntok - 1), wp1 = base + q0 + min(wave * 32 + 31, ntok - 1);
  const int w_lo = window_start(a.window, wp0), w_in = window_start(a.window, wp1);

  int qpos[2], first[2];
  Run st[2];
  bf16x8 qf[2][DK / 32];
#pragma unroll
  for (int t = 0; t < 2; ++t) {
    const int tok = q0 + min(wave * 32 + t * 16 + fr, ntok - 1);
    qpos[t] = base + tok;
    first[t] = window_start(a.window, qpos[t]);
    st[t] = {-INFINITY, 0.f};
    const bf16* zp = (const bf16*)a.z + (size_t)(qs + tok) * a.ldz + h * (a.dim + a.rot);
    const float* cs = a.cos_sin + (size_t)a.pos[qs + tok] * a.pairs * 2;
#pragma unroll
    for (int ks = 0; ks < DK / 32; ++ks) {
      const int d = ks * 32 + fq * 8;
      if (ks * 32 < a.dim) {                             // (dim % 32 == 0)
        qf[t][ks] = *reinterpret_cast<const bf16x8*>(zp + d);
      } else {
        float v[8] = {};
        if (d - a.dim < a.rot) rotated8(zp + a.dim, cs, a.pairs, a.rot, d - a.dim, v);
#pragma unroll
        for (int j = 0; j < 8; ++j) qf[t][ks][j] = (bf16)v[j];
      }
    }
  }
  ScoreConst kc = {a.scale * LOG2E, 0.f, 0.f};
  f32x4 o[2][DV / 16];
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int i = 0; i < DV / 16; ++i) o[t][i] = f32x4{0.f, 0.f, 0.f, 0.f};

  const int* bt = a.block_table + (size_t)s * a.max_blocks;
  const bf16* ex = (const bf16*)a.exp + (long long)a.key0[s] * a.lde + (size_t)h * (a.dim + DV);
  // lane offsets (bytes) of the DMA pieces, which repeat every 8 rows.  Keys: the
  // expanded part, then the shared rotated part (past it whatever is finite: the
  // query is zero there); values follow the expanded key part
  unsigned koff[DK / 64], voff[DV / 64];
  bool rot_j[DK / 64];
#pragma unroll
  for (int j = 0; j < DK / 64; ++j) {
    const int c = j * 64 + lane, row = c / (DK / 8), d = ((c % (DK / 8)) ^ (row & 7)) << 3, dr = d - a.dim;
    rot_j[j] = dr >= 0;
    koff[j] = 2 * (dr >= 0 ? row * a.ldc + (dr < a.rot ? dr : 0) : row * (int)a.lde + d);
  }
#pragma unroll
  for (int j = 0; j < DV / 64; ++j) {
    const int c = j * 64 + lane, row = c / (DV / 8), d = ((c % (DV / 8)) ^ (row & 7)) << 3;
    voff[j] = 2 * (row * (int)a.lde + a.dim + d);
  }
  const KeyFrag<DK> kfrag(Kl, fr, fq);
  const ValFrag<DV> vfrag(Vl, lane);
  const int kt0 = b_lo / KT, kt1 = b_hi / KT;
  int bt_v = 0;
  for (int kt = kt0; kt <= kt1; ++kt) {
    if (((kt - kt0) & 63) == 0) bt_v = kt + lane <= kt1 ? bt[kt + lane] : 0;   // 64 table entries per load
    const int blk = __builtin_amdgcn_readlane(bt_v, (kt - kt0) & 63);
    const bf16* er = ex + (long long)kt * KT * a.lde;
    const bf16* rr = (const bf16*)a.cache + (size_t)blk * KT * a.ldc + a.rank;
#pragma unroll
    for (int i = 0; i < DK / 32; ++i) {
      const int j = i % (DK / 64), down = wave * 16 + i / (DK / 64) * 8;   // the piece's pattern and first row
      const char* src = rot_j[j] ? (const char*)rr + (size_t)down * a.ldc * 2
                                 : (const char*)er + (size_t)down * a.lde * 2;
      glds16(src + koff[j], Kl + (wave * (DK / 32) + i) * 512);
    }
#pragma unroll
    for (int i = 0; i < DV / 32; ++i) {
      const int j = i % (DV / 64), down = wave * 16 + i / (DV / 64) * 8;
      glds16((const char*)er + (size_t)down * a.lde * 2 + voff[j], Vl + (wave * (DV / 32) + i) * 512);
    }
    __syncthreads();                                     // drains the LDS-DMA
    const int k_lo = kt * KT, k_hi = k_lo + KT - 1;
    if (w_on && k_lo <= wp1 && k_hi >= w_lo) {           // (wave-uniform) some row of the wave sees it
      f32x4 sacc[2][4];
#pragma unroll
      for (int nt = 0; nt < 4; ++nt) {
        sacc[0][nt] = sacc[1][nt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < DK / 32; ++ks) {
          const bf16x8 kf = kfrag.at(nt * 16, ks);
          sacc[0][nt] = mfma16x16x32(kf, qf[0][ks], sacc[0][nt]);
          sacc[1][nt] = mfma16x16x32(kf, qf[1][ks], sacc[1][nt]);
        }
      }
      bf16x8 pf[2][2];
      const bool inside = k_hi <= wp0 && k_lo >= w_in;
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const int lo = first[t] - k_lo, hi = qpos[t] - k_lo;
        const float alpha = inside ? tile_weights<PLAIN, false>(sacc[t], pf[t], st[t], kc, lo, hi, -KT, fq)
                                   : tile_weights<PLAIN, true>(sacc[t], pf[t], st[t], kc, lo, hi, -KT, fq);
        if (__any(alpha != 1.f)) {
#pragma unroll
          for (int dt = 0; dt < DV / 16; ++dt) o[t][dt] *= alpha;
        }
      }
#pragma unroll
      for (int dt = 0; dt < DV / 16; ++dt)
#pragma unroll
        for (int k2 = 0; k2 < 2; ++k2) {
          const bf16x8 vf = vfrag.at(dt & 3, k2, (dt >> 2) * 64);
          o[0][dt] = mfma16x16x32(vf, pf[0][k2], o[0][dt]);
          o[1][dt] = mfma16x16x32(vf, pf[1][k2], o[1][dt]);
        }
    }
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < 2; ++t) {
    float l = st[t].l + __shfl_xor(st[t].l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    const int row = wave * 32 + t * 16 + fr;
    if (row >= ntok) continue;
    const size_t tok = (size_t)qs + q0 + row;
    const float inv = l > 0.f ? head_gate<bf16>(a, tok, h) / l : 0.f;
    bf16* op = (bf16*)a.out + (tok * a.H + h) * DV + 4 * fq;
#pragma unroll
    for (int dt = 0; dt < DV / 16; ++dt) {
      bf16x4 w;
#pragma unroll
      for (int r = 0; r < 4; ++r) w[r] = (bf16)(o[t][dt][r] * inv);
      *reinterpret_cast<bf16x4*>(op + dt * 16) = w;
    }
  }
}

template <int DK>
int launch_prefill_dk(const LatentPrefillArgs& a, hipStream_t s) {
  const dim3 grid(a.H, a.items);
  switch (a.DV) {
    case 64: attn_latent_prefill_kernel<DK, 64><<<grid, 256, 0, s>>>(a); return 0;
    case 128: attn_latent_prefill_kernel<DK, 128><<<grid, 256, 0, s>>>(a); return 0;
    case 192: attn_latent_prefill_kernel<DK, 192><<<grid, 256, 0, s>>>(a); return 0;
    case 256: attn_latent_prefill_kernel<DK, 256><<<grid, 256, 0, s>>>(a); return 0;
    default: return 3;
  }
}

}  // namespace

// One work list; 3: a (DK, DV) pair without a kernel (the row form takes it)
int launch_attn_latent(const MaskedAttnArgs& a, int nwork, int form, int nz, hipStream_t s) {
  if (nwork <= 0) return 0;
  if (a.Hkv != 1 || a.cap > 0.f || a.slopes) return 1;
  if (nz < 1 || nz > MAX_SPLITS || (nz > 1 && (!a.split_o || !a.split_ml))) return 2;
  switch (a.DK * 1024 + a.DV) {
    case 64 * 1024 + 64: return launch_pair<64, 64>(a, nwork, form, nz, s);
    case 128 * 1024 + 64: return launch_pair<128, 64>(a, nwork, form, nz, s);
    case 128 * 1024 + 128: return launch_pair<128, 128>(a, nwork, form, nz, s);
    case 192 * 1024 + 128: return launch_pair<192, 128>(a, nwork, form, nz, s);
    case 192 * 1024 + 192: return launch_pair<192, 192>(a, nwork, form, nz, s);
    case 256 * 1024 + 192: return launch_pair<256, 192>(a, nwork, form, nz, s);
    case 256 * 1024 + 256: return launch_pair<256, 256>(a, nwork, form, nz, s);
    case 320 * 1024 + 256: return launch_pair<320, 256>(a, nwork, form, nz, s);
    case 448 * 1024 + 384: return launch_pair<448, 384>(a, nwork, form, nz, s);
    case 576 * 1024 + 512: return launch_pair<576, 512>(a, nwork, form, nz, s);
    default: return 3;
  }
}

int launch_attn_latent_prefill(const LatentPrefillArgs& a, hipStream_t s) {
  if (a.items <= 0) return 0;
  if (a.dim % 32 || a.rot % 8 || a.dim + a.rot > a.DK || a.items > 65535 || 2 * a.pairs > a.rot) return 1;
  switch (a.DK) {
    case 64: return launch_prefill_dk<64>(a, s);
    case 128: return launch_prefill_dk<128>(a, s);
    case 192: return launch_prefill_dk<192>(a, s);
    case 256: return launch_prefill_dk<256>(a, s);
    default: return 3;
  }
}
