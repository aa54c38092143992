// Shared by the masked attention kernels: what they know about scores and cached
// rows, the tiles of a packed step, matrix-core fragments, base-2 scores.
#pragma once

#include "seq_common.h"

constexpr float kLog2e = 1.4426950408889634f;

// What every attention kernel needs to know about scores and rows.
// Visible keys of position p: [0, kept(p)) and [lower(p), p].
struct AttnArgs {
  float scale, softcap, out_scale;
  int chunk, window, keep;
  const float* sink;    // [H] or null: score of a key without a value
  const float* slopes;  // [H] or null: slopes[h] * (i - j) comes off a score
  const float* kscale;  // [blocks, bs] or null: factor of a cached key's scores
  const void* gate;     // [T, H] or null: head h's output times sigmoid(gate[t, h])
  int64_t gate_rs;      // elements between gate rows
  int64_t v_rs;         // elements between value rows
  int H, G, D, Dv, bs, kvs;
  int bs_shift;         // log2 of bs, or -1

  DEV_INLINE int lower(int p) const {
    int lo = 0;
    if (chunk > 0) lo = (p / chunk) * chunk;
    if (window > 0) lo = max(lo, p - window + 1);
    return lo;
  }
  DEV_INLINE int kept(int lo) const { return min(keep, lo); }
  // factor of head h's output at token t; gate holds elements of type T
  template <typename T>
  DEV_INLINE float out_factor(int t, int h) const {
    if (gate == nullptr) return out_scale;
    return out_scale * sigmoid_f(ldf((const T*)gate + (size_t)t * gate_rs + h));
  }
};

// softcap * tanh(x / softcap) times log2 e as cap2 - 2 cap2 / (e^(2x/cap) + 1):
// absolute error below 1e-6 of the cap. x comes multiplied by 2 log2(e) / cap.
DEV_INLINE float cap_base2(float x, float cap2) {
  return cap2 - 2.f * cap2 * __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(x) + 1.f);
}

typedef __attribute__((ext_vector_type(4))) short bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

// two fp32 -> packed bf16 pair (round to nearest even), low half first; a
// conversion the compiler knows, so that it keeps the wait states between an
// exponential and its reader
typedef __attribute__((ext_vector_type(2))) float f32x2;
typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
DEV_INLINE uint32_t cvt_pk_bf16(float a, float b) {
  return __builtin_bit_cast(uint32_t, __builtin_convertvector((f32x2){a, b}, bf16x2));
}

// max over the four lanes 16 apart that share a lane column
DEV_INLINE float column_max(float x, int lane) {
  auto from = [&](float v, int src) {
    return __builtin_bit_cast(
        float, __builtin_amdgcn_ds_bpermute(src * 4, __builtin_bit_cast(int, v)));
  };
  x = fmaxf(x, from(x, lane ^ 16));
  return fmaxf(x, from(x, lane ^ 32));
}

constexpr int kKT = 32;    // keys of a tile
constexpr int kRPad = 8;   // padding of a staged row (elements)

typedef __attribute__((ext_vector_type(8))) short bf16x8;

// A 16 x 16 piece of a row-major LDS tile, transposed on the way to the
// registers: p points at (row r0 + (lane & 15) / 4 + 4 * (lane >> 4), column
// c0 + 4 * (lane & 3)); the lane receives rows r0 + 4 * (lane >> 4) + 0..3 of
// column c0 + (lane & 15).
DEV_INLINE bf16x4 lds_read_transposed(const bf16raw* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) bf16x4*)p);
}

// K Q^T over 16 (four slots a lane) or 32 (eight slots) key dims
DEV_INLINE f32x4 mfma_qk(bf16x4 k, bf16x4 q, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(k, q, c, 0, 0, 0);
}
DEV_INLINE f32x4 mfma_qk(bf16x8 k, bf16x8 q, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, q, c, 0, 0, 0);
}

template <bool kWide> struct QkFrag {  // one lane's share of a row step
  typedef bf16x4 type;
  static constexpr int kDims = 16, kElems = 4;
};
template <> struct QkFrag<true> {
  typedef bf16x8 type;
  static constexpr int kDims = 32, kElems = 8;
};

// Per-head constants of a score in the base-2 domain (score * log2 e, so that
// every exponential is one v_exp_f32).
struct ScoreConsts {
  float mul;    // on the dot product: scale, with a cap times 2 log2(e) / cap
  float cap2;   // cap * log2 e, or 0
  float slope2; // slope * log2 e, or 0
  DEV_INLINE ScoreConsts(const AttnArgs& a, int h) {
    mul = a.softcap > 0.f ? a.scale * (2.f * kLog2e) / a.softcap : a.scale * kLog2e;
    cap2 = a.softcap * kLog2e;
    slope2 = a.slopes != nullptr ? a.slopes[h] * kLog2e : 0.f;
  }
};

// Scores of a lane's eight keys of a 32-key tile (keys sub * 16 + grp * 4 + i,
// e = sub * 4 + i): scale and key scale, cap, bias. rel0 = (the lane's first
// key - query). kcv: the tile's key scales in LDS at the lane's keys, or null.
template <bool kBias>
DEV_INLINE void base2_scores(const f32x4* sacc, const ScoreConsts& k, float rel0,
                             const float* kcv, float* sc) {
  if (kcv != nullptr) {
    const float4 k0 = *(const float4*)kcv, k1 = *(const float4*)(kcv + 16);
    sc[0] = sacc[0][0] * (k.mul * k0.x); sc[1] = sacc[0][1] * (k.mul * k0.y);
    sc[2] = sacc[0][2] * (k.mul * k0.z); sc[3] = sacc[0][3] * (k.mul * k0.w);
    sc[4] = sacc[1][0] * (k.mul * k1.x); sc[5] = sacc[1][1] * (k.mul * k1.y);
    sc[6] = sacc[1][2] * (k.mul * k1.z); sc[7] = sacc[1][3] * (k.mul * k1.w);
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) sc[e] = sacc[e >> 2][e & 3] * k.mul;
  }
  if (k.cap2 > 0.f) {
#pragma unroll
    for (int e = 0; e < 8; ++e) sc[e] = cap_base2(sc[e], k.cap2);
  }
  if (kBias) {
    const float b = k.slope2 * rel0;
#pragma unroll
    for (int e = 0; e < 8; ++e) sc[e] += fmaf(k.slope2, (float)((e >> 2) * 16 + (e & 3)), b);
  }
}

