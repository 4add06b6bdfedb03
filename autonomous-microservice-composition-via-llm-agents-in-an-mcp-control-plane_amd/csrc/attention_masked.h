// Device parts of the masked attention forms (attention_masked.hip,
// attention_latent.hip): scores, masks, softmax weights of a 64-key tile, P V.
#pragma once
#include "common.h"
#include "kernels.h"

namespace {

constexpr int KT = 64;                        // keys per cache block

typedef __attribute__((ext_vector_type(4))) short s16x4;
constexpr float LOG2E = 1.4426950408889634f;
constexpr float NOMAX_CAP = 60.f;             // e^60 x 1e6 keys is far below fp32's range

enum { PLAIN = 0, CAPPED = 1, CAPPED_NOMAX = 2, BIASED = 3 };   // score forms

DEV bf16x4 tr_read(const bf16* p) {
  s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(p));
  return __builtin_bit_cast(bf16x4, v);
}

// Score constants (log2 units): PLAIN s = acc a; BIASED s = acc a - b distance, b
// the row's slope; CAPPED s = C tanh(acc scale / cap)
// = C - 2 C / (1 + 2^(acc a)), a = 2 log2(e) scale / cap, C = cap log2(e)
struct ScoreConst {
  float a, c, b;
};
template <int MODE>
DEV ScoreConst score_const(const MaskedAttnArgs& p, int head) {
  if constexpr (MODE == PLAIN) return {p.scale * LOG2E, 0.f, 0.f};
  if constexpr (MODE == BIASED) return {p.scale * LOG2E, 0.f, p.slopes[head] * LOG2E};
  return {2.f * LOG2E * p.scale / p.cap, p.cap * LOG2E, 0.f};
}
template <int MODE>
DEV float score(float acc, const ScoreConst& k, float bias) {
  if constexpr (MODE == PLAIN) return acc * k.a;
  if constexpr (MODE == BIASED) return fmaf(acc, k.a, bias);
  return fmaf(-2.f * k.c, __builtin_amdgcn_rcpf(1.f + fexp2(acc * k.a)), k.c);
}

// running softmax state of one query row (the lane's)
struct Run {
  float m, l;                                 // maximum (log2 units; 0 in CAPPED_NOMAX), this lane's sum
};
// at the start: nothing, or (``sink``) the sink's score and its weight of one
template <int MODE>
DEV Run run_start(const MaskedAttnArgs& p, int head, bool sink, int fq) {
  const float s0 = sink && p.sinks ? p.sinks[head] * LOG2E : 0.f;
  if constexpr (MODE == CAPPED_NOMAX) return {0.f, sink && fq == 0 ? fexp2(s0) : 0.f};
  return {sink ? s0 : -INFINITY, sink && fq == 0 ? 1.f : 0.f};
}

// the output factor of a row
template <class T, class Args>
DEV float head_gate(const Args& p, size_t tok, int head) {
  if (!p.gate) return 1.f;
  const float z = (float)((const T*)p.gate)[tok * p.gate_ld + head];
  return 1.f / (1.f + expf(-z));
}

// One 64-key tile of the lane's row (keys 16 nt + 4 fq + r): scores -> weights
// (bf16 MFMA fragments, key order as in the accumulators).  lo, hi, keep are
// tile-relative; hi is the row's own position.  MASKED: keys after hi, and those
// before lo that are not before keep, drop out.  Returns the factor O is to be
// rescaled by.
template <int MODE, bool MASKED>
DEV float tile_weights(f32x4 (&sacc)[4], bf16x8 (&pf)[2], Run& st, const ScoreConst& k, int lo, int hi,
                       int keep, int fq) {
  float alpha = 1.f;
  float tmax = -INFINITY;
  const float b0 = -k.b * (float)(hi - fq * 4);      // the lane's first key
#pragma unroll
  for (int nt = 0; nt < 4; ++nt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float v = score<MODE>(sacc[nt][r], k, fmaf(k.b, (float)(nt * 16 + r), b0));
      if constexpr (MASKED) {
        const int key = nt * 16 + fq * 4 + r;
        v = (key <= hi && (key >= lo || key < keep)) ? v : -INFINITY;
      }
      sacc[nt][r] = v;
      if constexpr (MODE != CAPPED_NOMAX) tmax = fmaxf(tmax, v);
    }
  float mu = 0.f;
  if constexpr (MODE != CAPPED_NOMAX) {
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float m_new = fmaxf(st.m, tmax);
    mu = m_new == -INFINITY ? 0.f : m_new;    // every key masked so far
    alpha = fexp2(st.m - mu);
    st.m = m_new;
  }
  float sum = 0.f;
#pragma unroll
  for (int nt = 0; nt < 4; ++nt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float p = fexp2(sacc[nt][r] - mu);
      sum += p;
      pf[nt >> 1][(nt & 1) * 4 + r] = (bf16)p;
    }
  st.l = st.l * alpha + sum;
  return alpha;
}

// Addresses of a lane's fragments in a [64][LD] tile whose 16-B chunks are swizzled
// by row & 7.  The swizzle only touches the low three bits of a chunk, so a few bases
// and constant offsets reach everything.
template <int LD>
struct KeyFrag {                              // rows of K as MFMA operands
  const bf16* p[2];
  DEV KeyFrag(const bf16* Kl, int row, int fq) {
#pragma unroll
    for (int j = 0; j < 2; ++j) p[j] = Kl + row * LD + (((j * 4 + fq) ^ (row & 7)) << 3);
  }
  // 32 columns ``ks`` of a row ``down`` (a multiple of 8) below
  DEV bf16x8 at(int down, int ks) const {
    return *reinterpret_cast<const bf16x8*>(p[ks & 1] + down * LD + (ks >> 1) * 64);
  }
};
template <int LD, int NB = 4>
struct ValFrag {                              // V^T through transposed reads
  const bf16* p[NB];                          // 16-column tiles dt0 + 0 .. NB - 1 (mod 4)
  DEV ValFrag(const bf16* Vl, int lane, int dt0 = 0) {
    const int key = (lane >> 4) * 4 + ((lane & 15) >> 2), tp = lane & 3;
#pragma unroll
    for (int j = 0; j < NB; ++j)
      p[j] = Vl + key * LD + (((((dt0 + j) & 3) * 2 + (tp >> 1)) ^ (key & 7)) << 3) + (tp & 1) * 4;
  }
  // keys 32 k2 + 4 fq .. + 3 and 16 further, base j, ``cols`` (a multiple of 64) columns on
  DEV bf16x8 at(int j, int k2, int cols) const {
    const bf16* q = p[j] + k2 * 32 * LD + cols;
    const bf16x4 v0 = tr_read(q), v1 = tr_read(q + 16 * LD);
    return bf16x8{v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
  }
};

// O^T += V^T P^T over one tile; Vl: [64][DV] with 16-B chunk swizzle ^= row & 7
template <int DV>
DEV void tile_pv(const bf16* Vl, const bf16x8 (&pf)[2], f32x4 (&o)[DV / 16], int lane) {
  const ValFrag<DV> vf(Vl, lane);
#pragma unroll
  for (int dt = 0; dt < DV / 16; ++dt)
#pragma unroll
    for (int k2 = 0; k2 < 2; ++k2) o[dt] = mfma16x16x32(vf.at(dt & 3, k2, (dt >> 2) * 64), pf[k2], o[dt]);
}

// LDS-DMA of pieces [first, first + P1) (1 KiB each) of a [64][D] block, swizzled;
// D / 64 pieces are 8 rows, so their lane offsets repeat from there
template <int D, int P0, int P1>
DEV void stage_rows(const bf16* src, bf16* dst, int first, int lane) {
  constexpr int NC = D / 8, M = D / 64;       // 16-B chunks per row, pieces per 8 rows
  if constexpr (P1 % M == 0 && P0 == 0) {     // whole 8-row groups (``first`` is one, too)
    const char* base = (const char*)(src + (first / M) * 8 * D);
    unsigned off[M];
#pragma unroll
    for (int j = 0; j < M; ++j) {
      const int c = j * 64 + lane, row = c / NC, chunk = c % NC;
      off[j] = (row * D + ((chunk ^ (row & 7)) << 3)) * 2;
    }
#pragma unroll
    for (int i = 0; i < P1; ++i)
      glds16(base + (i / M) * 8 * D * 2 + off[i % M], dst + (first + i) * 512);
  } else {
#pragma unroll
    for (int i = P0; i < P1; ++i) {
      const int p = first + i;
      const int c = p * 64 + lane;
      const int row = c / NC, chunk = c % NC;
      glds16(src + row * D + ((chunk ^ (row & 7)) << 3), dst + p * 512);
    }
  }
}

// first key a query at ``pos`` sees (apart from the kept first ones)
DEV int window_start(int window, int pos) { return window > 0 ? max(pos - window + 1, 0) : 0; }
DEV int first_key(const MaskedAttnArgs& p, int pos) {
  return p.chunk > 0 ? pos / p.chunk * p.chunk : window_start(p.window, pos);
}

// key tiles of rows whose first keys start at ``lo`` and whose last position is
// ``hi``: those that hold kept first keys, then lo / KT .. hi / KT
struct TileWalk {
  int kept, lo, n;
  DEV TileWalk(const MaskedAttnArgs& p, int lo_key, int hi_key) {
    lo = lo_key / KT;
    kept = min((p.keep + KT - 1) / KT, lo);
    n = kept + hi_key / KT - lo + 1;
  }
  DEV int tile(int i) const { return i < kept ? i : lo + i - kept; }
};

}  // namespace
