// Rotary (interleaved pairs, or split halves after a whole-row RMS norm of q
// and k) fused with the paged cache write, and softmax attention of every
// packed token over its own sequence's cached keys under a chunk / window
// mask, with separate key and value sizes. Options: first tokens that stay
// visible behind a window, a tanh cap, a bias per position, a scale per cached
// key, a sink (a score without a value: one more term in the denominator), and
// a sigmoid gate per token and head on the output.
#include "attn_masked.h"

#include <type_traits>

// Single decode tokens on the matrix cores (attention_masked_decode.hip); false
// when the sizes are not its.
bool masked_decode_mfma(const torch::Tensor& out, const torch::Tensor& q,
                        const torch::Tensor& k_cache, const torch::Tensor& v_cache,
                        const torch::Tensor& block_tables, const torch::Tensor& token_seq,
                        const torch::Tensor& positions, const AttnArgs& args, bool tied);

namespace {

// grid (T): q pairs rotate in place; k pairs rotate into the key cache;
// v copies into the value cache. Angles are fp32: position * inv_freq[i].
template <typename T>
__global__ void rope_pairs_cache_kernel(
    T* __restrict__ q, int64_t q_stride, const T* __restrict__ k,
    int64_t k_stride, const T* __restrict__ v, int64_t v_stride,
    const int* __restrict__ positions, const float* __restrict__ inv_freq,
    int half, T* __restrict__ k_cache, T* __restrict__ v_cache,
    const int64_t* __restrict__ slot_mapping, int H, int G, int D, int Dv,
    int bs) {
  const int t = blockIdx.x;
  const float pos = (float)positions[t];
  const int64_t slot = slot_mapping[t];
  const int hp = D / 2;
  const int nqp = H * hp, nkp = G * hp, nv = G * Dv;
  const int64_t blk = slot >= 0 ? slot / bs : 0;
  const int off = slot >= 0 ? (int)(slot % bs) : 0;
  for (int u = threadIdx.x; u < nqp + nkp + nv; u += blockDim.x) {
    if (u < nqp + nkp) {
      const bool is_q = u < nqp;
      const int uu = is_q ? u : u - nqp;
      const int hd = uu / hp, i = uu % hp;
      const T* src = is_q ? q + (size_t)t * q_stride + hd * D + 2 * i
                          : k + (size_t)t * k_stride + hd * D + 2 * i;
      float a = ldf(src), b = ldf(src + 1);
      if (i < half) {
        float sn, cs;
        sincosf(pos * inv_freq[i], &sn, &cs);
        const float ra = a * cs - b * sn, rb = b * cs + a * sn;
        a = ra;
        b = rb;
      }
      if (is_q) {
        if (i < half) {
          T* dst = q + (size_t)t * q_stride + hd * D + 2 * i;
          stf(dst, a);
          stf(dst + 1, b);
        }
      } else if (slot >= 0) {
        T* dst = k_cache + (((size_t)blk * G + hd) * bs + off) * D + 2 * i;
        stf(dst, a);
        stf(dst + 1, b);
      }
    } else if (slot >= 0) {
      const int e = u - nqp - nkp;
      const int g = e / Dv, d = e % Dv;
      v_cache[(((size_t)blk * G + g) * bs + off) * Dv + d] =
          v[(size_t)t * v_stride + g * Dv + d];
    }
  }
}

// grid (T). q and k rows are RMS-normed as a whole (all heads at once, plain
// weights), then the first 2 * half dims of every head rotate with dimension
// i paired with i + half; the rest pass. q is rewritten in place, k goes to
// the key cache, v is copied to the value cache. fp32 throughout.
template <typename T>
__global__ __launch_bounds__(256) void qknorm_rope_half_cache_kernel(
    T* __restrict__ q, int64_t q_stride, const T* __restrict__ k,
    int64_t k_stride, const T* __restrict__ v, int64_t v_stride,
    const float* __restrict__ qw, const float* __restrict__ kw, float eps,
    const int* __restrict__ positions, const float* __restrict__ inv_freq,
    int half, T* __restrict__ k_cache, T* __restrict__ v_cache,
    const int64_t* __restrict__ slot_mapping, int H, int G, int D, int Dv,
    int bs) {
  __shared__ float red0[16], red1[16];
  const int t = blockIdx.x;
  const float pos = (float)positions[t];
  const int64_t slot = slot_mapping[t];
  T* qr = q + (size_t)t * q_stride;
  const T* kr = k + (size_t)t * k_stride;
  float rq = 1.f, rk = 1.f;
  if (qw != nullptr) {
    float sq = 0.f, sk = 0.f;
    for (int i = threadIdx.x; i < H * D; i += blockDim.x) {
      const float x = ldf(qr + i);
      sq += x * x;
    }
    for (int i = threadIdx.x; i < G * D; i += blockDim.x) {
      const float x = ldf(kr + i);
      sk += x * x;
    }
    rq = 1.0f / sqrtf(block_sum(sq, red0) / (float)(H * D) + eps);
    rk = 1.0f / sqrtf(block_sum(sk, red1) / (float)(G * D) + eps);
  }
  const int upr = D - half;  // units per head: `half` pairs, then single dims
  const int nq = H * upr, nk = G * upr, nv = G * Dv;
  const int64_t blk = slot >= 0 ? slot / bs : 0;
  const int off = slot >= 0 ? (int)(slot % bs) : 0;
  for (int u = threadIdx.x; u < nq + nk + nv; u += blockDim.x) {
    if (u < nq + nk) {
      const bool is_q = u < nq;
      const int uu = is_q ? u : u - nq;
      const int hd = uu / upr, i = uu % upr;
      if (!is_q && slot < 0) continue;
      const T* src = is_q ? qr + hd * D : kr + hd * D;
      const float* w = is_q ? qw : kw;
      const float r = is_q ? rq : rk;
      T* dst = is_q ? qr + hd * D
                    : k_cache + (((size_t)blk * G + hd) * bs + off) * D;
      if (i < half) {
        float a = ldf(src + i) * r, b = ldf(src + i + half) * r;
        if (w != nullptr) {
          a *= w[hd * D + i];
          b *= w[hd * D + i + half];
        }
        float sn, cs;
        sincosf(pos * inv_freq[i], &sn, &cs);
        stf(dst + i, a * cs - b * sn);
        stf(dst + i + half, b * cs + a * sn);
      } else {
        const int d = i + half;
        float a = ldf(src + d) * r;
        if (w != nullptr) a *= w[hd * D + d];
        stf(dst + d, a);
      }
    } else if (slot >= 0) {
      const int e = u - nq - nk;
      const int g = e / Dv, d = e % Dv;
      v_cache[(((size_t)blk * G + g) * bs + off) * Dv + d] =
          v[(size_t)t * v_stride + g * Dv + d];
    }
  }
}

// grid (T). Whole-row RMS norms of q and k when a cached row is key and value:
// q <- q / rms(q) * w in place; k's row goes to the cache as it is and
// 1 / rms(k) to key_scale. kVec: 16-byte accesses (rows and heads of whole,
// aligned vectors).
template <typename T, bool kVec>
__global__ __launch_bounds__(256) void qnorm_rows_cache_kernel(
    T* __restrict__ q, int64_t q_stride, const T* __restrict__ k, int64_t k_stride,
    const float* __restrict__ w, float eps, T* __restrict__ cache,
    float* __restrict__ key_scale, const int64_t* __restrict__ slot_mapping, int H,
    int G, int D, int bs) {
  constexpr int N = kVec ? Vec16<T>::N : 1;
  __shared__ float red0[16], red1[16];
  const int t = blockIdx.x;
  const int64_t slot = slot_mapping[t];
  T* qr = q + (size_t)t * q_stride;
  const T* kr = k + (size_t)t * k_stride;
  const int nq = H * D, nk = G * D;
  auto load = [](const T* p, float* x) {
    if constexpr (kVec) Vec16<T>::load(p, x);
    else x[0] = ldf(p);
  };
  float sq = 0.f, sk = 0.f;
  for (int i = threadIdx.x * N; i < nq; i += blockDim.x * N) {
    float x[N];
    load(qr + i, x);
#pragma unroll
    for (int e = 0; e < N; ++e) sq += x[e] * x[e];
  }
  const int64_t blk = slot >= 0 ? slot / bs : 0;
  const int off = slot >= 0 ? (int)(slot % bs) : 0;
  for (int i = threadIdx.x * N; i < nk; i += blockDim.x * N) {
    float x[N];
    load(kr + i, x);
#pragma unroll
    for (int e = 0; e < N; ++e) sk += x[e] * x[e];
    if (slot >= 0) {
      const int g = i / D, d = i % D;
      T* dst = cache + (((size_t)blk * G + g) * bs + off) * D + d;
      if constexpr (kVec) *(uint4*)dst = *(const uint4*)(kr + i);
      else *dst = kr[i];
    }
  }
  const float rq = 1.0f / sqrtf(block_sum(sq, red0) / (float)nq + eps);
  const float rk = 1.0f / sqrtf(block_sum(sk, red1) / (float)nk + eps);
  if (slot >= 0 && threadIdx.x == 0) key_scale[slot] = rk;
  for (int i = threadIdx.x * N; i < nq; i += blockDim.x * N) {
    float x[N];
    load(qr + i, x);
#pragma unroll
    for (int e = 0; e < N; ++e) x[e] *= rq * w[i + e];
    if constexpr (kVec) Vec16<T>::store(qr + i, x);
    else stf(qr + i, x[0]);
  }
}

// grid (T), 256 threads. RMS norm of every q and k head by itself, without a
// weight (q in place, k into the key cache), v copied to the value cache. kVec:
// `lpr` neighbouring lanes (a power of two) own a head's row, a 16-byte piece
// each; otherwise a wave owns it. fp32 inside.
template <typename T, bool kVec>
__global__ __launch_bounds__(256) void headnorm_qk_cache_kernel(
    T* __restrict__ q, int64_t q_stride, const T* __restrict__ k, int64_t k_stride,
    const T* __restrict__ v, int64_t v_stride, float eps, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const int64_t* __restrict__ slot_mapping, int H, int G,
    int D, int Dv, int bs, int lpr) {
  constexpr int N = kVec ? Vec16<T>::N : 1;
  const int t = blockIdx.x;
  const int64_t slot = slot_mapping[t];
  const int64_t blk = slot >= 0 ? slot / bs : 0;
  const int off = slot >= 0 ? (int)(slot % bs) : 0;
  const int per = kVec ? lpr : WAVE;  // lanes of a row
  const int lane = threadIdx.x % per, step = blockDim.x / per;
  const int n_rows = slot >= 0 ? H + G : H;
  // every lane of a wave walks the same number of rows: the shuffles need all
  for (int r0 = 0; r0 < n_rows; r0 += step) {
    const int row = r0 + threadIdx.x / per;
    const bool on = row < n_rows, is_q = row < H;
    const T* src = q;
    T* dst = q;
    if (on) {
      const int g = row - H;
      src = is_q ? q + (size_t)t * q_stride + row * D : k + (size_t)t * k_stride + g * D;
      dst = is_q ? q + (size_t)t * q_stride + row * D
                 : k_cache + (((size_t)blk * G + g) * bs + off) * D;
    }
    if constexpr (kVec) {
      float x[N];
      float ss = 0.f;
      const bool mine = on && lane * N < D;
      if (mine) {
        Vec16<T>::load(src + lane * N, x);
#pragma unroll
        for (int e = 0; e < N; ++e) ss += x[e] * x[e];
      }
      for (int o = lpr >> 1; o > 0; o >>= 1) ss += __shfl_xor(ss, o, WAVE);
      const float r = 1.0f / sqrtf(ss / (float)D + eps);
      if (mine) {
#pragma unroll
        for (int e = 0; e < N; ++e) x[e] *= r;
        Vec16<T>::store(dst + lane * N, x);
      }
    } else {
      float ss = 0.f;
      if (on)
        for (int d = lane; d < D; d += WAVE) {
          const float x = ldf(src + d);
          ss += x * x;
        }
      const float r = 1.0f / sqrtf(wave_sum(ss) / (float)D + eps);
      if (on)
        for (int d = lane; d < D; d += WAVE) stf(dst + d, ldf(src + d) * r);
    }
  }
  if (slot < 0) return;
  const T* vr = v + (size_t)t * v_stride;
  for (int i = threadIdx.x * N; i < G * Dv; i += blockDim.x * N) {
    const int g = i / Dv, d = i % Dv;
    T* dst = v_cache + (((size_t)blk * G + g) * bs + off) * Dv + d;
    if constexpr (kVec) *(uint4*)dst = *(const uint4*)(vr + i);
    else *dst = vr[i];
  }
}

constexpr int kMaxDvPerLane = 16;  // value size <= 1024
constexpr int kDecWaves = 4;

// grid (T, H), kDecWaves waves per (token, query head). Keys are walked in
// tiles of 64, dealt round-robin to the waves (a decode token alone cannot
// hide memory latency, so its keys are split): each lane scores one key
// (fp32 dot, cap, mask), the wave keeps a running max / sum, then its lanes
// turn to the values and accumulate p . V for the tile. The waves' partial
// results are joined through LDS at the end. Serves single decode tokens
// (and, in fp32 or at odd sizes, prompt portions): every token reads its
// keys, this step's included, from the cache.
//
// kVec: key and value rows are read with 16-byte loads. For the values a
// wave splits into 64 / (Dv / N) key groups, each lane owning N value
// channels of its group's keys.
template <typename T, bool kVec>
__global__ __launch_bounds__(kDecWaves * WAVE) void masked_paged_attention_kernel(
    T* __restrict__ out, int64_t out_stride, const T* __restrict__ q,
    int64_t q_stride, const T* __restrict__ k_cache,
    const T* __restrict__ v_cache, const int* __restrict__ block_tables,
    int max_blocks, const int* __restrict__ token_seq,
    const int* __restrict__ positions, AttnArgs a) {
  const int H = a.H, G = a.G, D = a.D, Dv = a.Dv, bs = a.bs;
  constexpr int N = Vec16<T>::N;
  const int lpr = kVec ? Dv / N : 1;          // lanes per value row
  const int ngrp = kVec ? WAVE / lpr : 1;     // key groups of a wave
  extern __shared__ float sm[];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  int64_t* vbase = (int64_t*)sm + wave * WAVE;       // [waves][64] value row offsets
  float* ps = sm + 2 * WAVE * kDecWaves + wave * WAVE;  // [waves][64] probabilities
  float* stat = sm + 3 * WAVE * kDecWaves;           // [waves][2] max, sum
  float* qs = stat + 2 * kDecWaves;                  // [D]
  float* red_all = qs + ((D + 3) & ~3);              // [waves][groups][Dv]
  float* red = red_all + (size_t)wave * ngrp * Dv;
  const int t = blockIdx.x, h = blockIdx.y;
  const int g = h / (H / G);
  const int pos = positions[t];
  const int* bt = block_tables + (size_t)token_seq[t] * max_blocks;
  // the visible keys are numbered 0 .. n_keys - 1: kept first tokens, then lo .. pos
  const int lo = a.lower(pos), kept = a.kept(lo), n_keys = kept + pos - lo + 1;
  const float slope = a.slopes != nullptr ? a.slopes[h] : 0.f;
  for (int i = threadIdx.x; i < D; i += blockDim.x)
    qs[i] = ldf(q + (size_t)t * q_stride + h * D + i);
  __syncthreads();
  const int kg = lane / lpr, lv = lane % lpr;
  const bool v_on = kVec && kg < ngrp;
  float m = -INFINITY, l = 0.f;
  float acc[kMaxDvPerLane];
#pragma unroll
  for (int i = 0; i < kMaxDvPerLane; ++i) acc[i] = 0.f;
  // the wave's own LDS rows are touched by this wave only, so the tile loop
  // needs no block barrier (a wave's LDS accesses complete in order)
  for (int v0 = wave * WAVE; v0 < n_keys; v0 += kDecWaves * WAVE) {
    const int vk = v0 + lane;
    float sc = -INFINITY;
    int64_t vb = 0;
    if (vk < n_keys) {
      const int j = vk < kept ? vk : lo + vk - kept;
      const int64_t blk = bt[j / bs];
      const int64_t rowi = (blk * G + g) * bs + (j % bs);
      const T* kp = k_cache + rowi * D;
      float dot = 0.f;
      if (kVec) {
        for (int i = 0; i < D; i += N) {
          float x[N];
          Vec16<T>::load(kp + i, x);
#pragma unroll
          for (int e = 0; e < N; ++e) dot += qs[i + e] * x[e];
        }
      } else {
        for (int i = 0; i < D; ++i) dot += qs[i] * ldf(kp + i);
      }
      sc = dot * a.scale;
      if (a.kscale != nullptr) sc *= a.kscale[blk * bs + j % bs];
      if (a.softcap > 0.f) sc = a.softcap * tanhf(sc / a.softcap);
      sc -= slope * (float)(pos - j);
      vb = ((blk * (G / a.kvs) + g / a.kvs) * bs + (j % bs)) * a.v_rs;
    }
    const float m_new = fmaxf(m, wave_max(sc));  // finite: lane 0's key is visible
    const float p = vk < n_keys ? expf(sc - m_new) : 0.f;
    const float corr = expf(m - m_new);  // m = -inf on the wave's first tile -> 0
    l = l * corr + wave_sum(p);
    m = m_new;
    ps[lane] = p;
    vbase[lane] = vb;
    __builtin_amdgcn_s_waitcnt(0xc07f);  // lgkmcnt(0): the wave's LDS writes landed
    __builtin_amdgcn_wave_barrier();
    const int nk = min(WAVE, n_keys - v0);
    if (kVec) {
#pragma unroll
      for (int e = 0; e < N; ++e) acc[e] *= corr;
      if (v_on) {
        for (int jj = kg; jj < nk; jj += ngrp) {
          float x[N];
          Vec16<T>::load(v_cache + vbase[jj] + lv * N, x);
          const float pj = ps[jj];
#pragma unroll
          for (int e = 0; e < N; ++e) acc[e] += pj * x[e];
        }
      }
    } else {
#pragma unroll
      for (int c = 0; c < kMaxDvPerLane; ++c) {
        const int d = c * WAVE + lane;
        if (d < Dv) {
          float x = acc[c] * corr;
          for (int jj = 0; jj < nk; ++jj) x += ps[jj] * ldf(v_cache + vbase[jj] + d);
          acc[c] = x;
        }
      }
    }
    __builtin_amdgcn_wave_barrier();  // all lanes read ps/vbase before the next tile
  }
  // join: every wave publishes (max, sum) and its unnormalised partial output
  if (lane == 0) {
    stat[2 * wave] = m;
    stat[2 * wave + 1] = l;
  }
  if (kVec) {
    if (v_on) {
#pragma unroll
      for (int e = 0; e < N; ++e) red[kg * Dv + lv * N + e] = acc[e];
    }
  } else {
#pragma unroll
    for (int c = 0; c < kMaxDvPerLane; ++c) {
      const int d = c * WAVE + lane;
      if (d < Dv) red[d] = acc[c];
    }
  }
  __syncthreads();
  float mx = -INFINITY;
  for (int w = 0; w < kDecWaves; ++w) mx = fmaxf(mx, stat[2 * w]);
  float wsc[kDecWaves], lsum = 0.f;
  for (int w = 0; w < kDecWaves; ++w) {
    const float mw = stat[2 * w];
    wsc[w] = mw == -INFINITY ? 0.f : expf(mw - mx);  // a wave may have had no tile
    lsum += stat[2 * w + 1] * wsc[w];
  }
  if (a.sink != nullptr) lsum += expf(a.sink[h] - mx);
  const float inv = a.out_factor<T>(t, h) / lsum;
  for (int d = threadIdx.x; d < Dv; d += blockDim.x) {
    float x = 0.f;
    for (int w = 0; w < kDecWaves; ++w) {
      const float* rw = red_all + (size_t)w * ngrp * Dv;
      float part = 0.f;
      for (int gi = 0; gi < ngrp; ++gi) part += rw[gi * Dv + d];
      x += part * wsc[w];
    }
    stf(out + (size_t)t * out_stride + h * Dv + d, x * inv);
  }
}

// Prompt portions on the matrix cores (bf16, key and value sizes multiples
// of 16). grid (query tiles, H), one wave per 16 consecutive
// queries of a run and one query head. Per 16-key tile:
//   S^T = K Q^T   (v_mfma_f32_16x16x16_bf16, K rows straight from the cache)
//   fp32 scale, cap, mask, running max / sum per query (a query is a lane
//   column, so its statistics never leave the lane quad 16 apart)
//   O^T += V^T P^T with P^T taken from S^T's accumulator layout as is.
// kMaxDSteps * 16 bounds the key size and kMaxDvTiles * 16 the value size
// (the query fragments and the output accumulators live in registers).
template <int kMaxDSteps, int kMaxDvTiles>
__global__ __launch_bounds__(WAVE) void masked_prefill_mfma_kernel(
    bf16raw* __restrict__ out, int64_t out_stride, const bf16raw* __restrict__ q,
    int64_t q_stride, const bf16raw* __restrict__ k_cache,
    const bf16raw* __restrict__ v_cache, const int* __restrict__ block_tables,
    int max_blocks, const int* __restrict__ start_loc,
    const int* __restrict__ positions, int n_seq, AttnArgs a) {
  const int H = a.H, G = a.G, D = a.D, Dv = a.Dv, bs = a.bs;
  int tile;
  const int s = find_tile(start_loc, n_seq, 16, blockIdx.x, &tile);
  const int h = blockIdx.y, g = h / (H / G);
  const int s0 = start_loc[s], s1 = start_loc[s + 1];
  const int q0 = s0 + tile * 16;
  if (q0 >= s1) return;
  const int nq = min(16, s1 - q0);
  const int lane = threadIdx.x, col = lane & 15, grp = lane >> 4;
  const bool q_ok = col < nq;
  const int tq = q0 + min(col, nq - 1);
  const int pos_q = q_ok ? positions[tq] : -1;
  const int pos_min = positions[q0], pos_max = pos_min + nq - 1;
  const int lo_q = q_ok ? a.lower(pos_q) : 0;
  const int lo_tile = a.lower(pos_min);
  // key tiles: those of the kept first tokens, then from the first query's
  // window to the last query
  const int kept = a.kept(lo_tile), n_kept = (kept + 15) / 16;
  const int n_tiles = n_kept + (pos_max - lo_tile) / 16 + 1;
  const float slope = a.slopes != nullptr ? a.slopes[h] : 0.f;
  const int* bt = block_tables + (size_t)s * max_blocks;
  const int nks = D / 16, ndt = Dv / 16;
  bf16x4 qf[kMaxDSteps];
#pragma unroll
  for (int ks = 0; ks < kMaxDSteps; ++ks)
    if (ks < nks)
      qf[ks] = *(const bf16x4*)(q + (size_t)tq * q_stride + h * D + ks * 16 + grp * 4);
  f32x4 oacc[kMaxDvTiles];
#pragma unroll
  for (int dt = 0; dt < kMaxDvTiles; ++dt) oacc[dt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  for (int it = 0; it < n_tiles; ++it) {
    const int j0 = it < n_kept ? it * 16 : lo_tile + (it - n_kept) * 16;
    const int j_end = it < n_kept ? kept - 1 : pos_max;
    // K operand: row = key j0 + col, 4 consecutive dims per step
    const int jk = min(j0 + col, j_end);
    const bf16raw* kp = k_cache + (((int64_t)bt[jk / bs] * G + g) * bs + jk % bs) * D + grp * 4;
    f32x4 sacc = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < kMaxDSteps; ++ks)
      if (ks < nks)
        sacc = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(
            *(const bf16x4*)(kp + ks * 16), qf[ks], sacc, 0, 0, 0);
    // this lane: query `col`, keys j0 + grp * 4 + i
    float sc[4];
    bool vis[4];
    int64_t vrow[4];
    float mt = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int j = j0 + grp * 4 + i;
      const int jv = min(j, j_end);
      const int64_t blk = bt[jv / bs];
      float x = sacc[i] * a.scale;
      if (a.kscale != nullptr) x *= a.kscale[blk * bs + jv % bs];
      if (a.softcap > 0.f) x = a.softcap * tanhf(x / a.softcap);
      x -= slope * (float)(pos_q - j);
      vis[i] = j <= j_end && j <= pos_q && (j >= lo_q || j < a.keep);
      sc[i] = vis[i] ? x : -INFINITY;
      mt = fmaxf(mt, sc[i]);
      vrow[i] = ((blk * (G / a.kvs) + g / a.kvs) * bs + jv % bs) * a.v_rs;
    }
    mt = fmaxf(mt, __shfl_xor(mt, 16, WAVE));
    mt = fmaxf(mt, __shfl_xor(mt, 32, WAVE));
    const float m_new = fmaxf(m, mt);
    const float corr = m_new == -INFINITY ? 1.f : expf(m - m_new);
    bf16x4 pb;
    float ps = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float p = vis[i] ? expf(sc[i] - m_new) : 0.f;
      ps += p;
      pb[i] = (short)f32_to_bf16(p);
    }
    l = l * corr + ps;
    m = m_new;
#pragma unroll
    for (int dt = 0; dt < kMaxDvTiles; ++dt) {
      if (dt < ndt) {
        bf16x4 vf;  // V^T operand: row = value dim dt*16 + col, keys grp*4 + i
#pragma unroll
        for (int i = 0; i < 4; ++i) vf[i] = (short)v_cache[vrow[i] + dt * 16 + col];
        f32x4 o = oacc[dt];
        o[0] *= corr; o[1] *= corr; o[2] *= corr; o[3] *= corr;
        oacc[dt] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(vf, pb, o, 0, 0, 0);
      }
    }
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (a.sink != nullptr) l += expf(a.sink[h] - m);
  if (q_ok) {
    const float inv = a.out_factor<bf16raw>(tq, h) / l;
    bf16raw* op = out + (size_t)tq * out_stride + h * Dv + grp * 4;
#pragma unroll
    for (int dt = 0; dt < kMaxDvTiles; ++dt) {
      if (dt < ndt) {
        ushort4 o4;
        o4.x = f32_to_bf16(oacc[dt][0] * inv);
        o4.y = f32_to_bf16(oacc[dt][1] * inv);
        o4.z = f32_to_bf16(oacc[dt][2] * inv);
        o4.w = f32_to_bf16(oacc[dt][3] * inv);
        *(ushort4*)(op + dt * 16) = o4;
      }
    }
  }
}

constexpr int kPrefillThreads = 512;

// Prompt portions on the matrix cores with the key / value tiles shared
// through LDS. A block of HW * QW waves covers QW * 16 consecutive queries of
// a run for HW query heads of one key/value head (for latent attention all
// heads share the one cached row, for grouped heads the group does). Per
// iteration the block stages 32 keys as they lie in the cache (16-byte loads,
// padded rows): K rows are read back as MFMA operands in 8 or 16-byte pieces,
// V rows through the transposing LDS read. kTied: the value is the leading
// part of the key row, so one staged tile serves both. Two LDS buffers: the
// next tile is loaded into registers before the products of the current one
// and written to the other buffer after them, one barrier per iteration. P V
// contracts all 32 keys of a tile in one v_mfma_f32_16x16x32_bf16 per 16 value
// dims (a lane's eight contraction slots are keys grp*4 + 0..3 and
// 16 + grp*4 + 0..3, for P and V alike), and so does K Q^T over 32 key dims
// when the key size allows (kWideQK). Statistics are fp32, base 2. kExact: the
// sizes are D = 16 kMaxDSteps, Dv = 16 kMaxDvTiles and the block size is a
// power of two; otherwise the template sizes are bounds and steps are guarded.
template <int kMaxDSteps, int kMaxDvTiles, bool kWideQK, bool kTied, bool kExact>
__global__ __launch_bounds__(kPrefillThreads) void masked_prefill_mfma_shared_kernel(
    bf16raw* __restrict__ out, int64_t out_stride, const bf16raw* __restrict__ q,
    int64_t q_stride, const bf16raw* __restrict__ k_cache,
    const bf16raw* __restrict__ v_cache, const int* __restrict__ block_tables,
    int max_blocks, const int* __restrict__ start_loc,
    const int* __restrict__ positions, int n_seq, int HW, int QW, AttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) bf16raw lds[];
  typedef QkFrag<kWideQK> Frag;
  typedef typename Frag::type frag_t;
  constexpr int kNF = kMaxDSteps * 16 / Frag::kDims;
  // 16-byte pieces of a tile per thread
  constexpr int nthr = kPrefillThreads;
  constexpr int kKVec = (kKT * kMaxDSteps * 2 + nthr - 1) / nthr;
  constexpr int kVVec = kTied ? 1 : (kKT * kMaxDvTiles * 2 + nthr - 1) / nthr;
  const int G = a.G;
  const int D = kExact ? kMaxDSteps * 16 : a.D, Dv = kExact ? kMaxDvTiles * 16 : a.Dv;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int col = lane & 15, grp = lane >> 4;
  const int hw = wave % HW, qw = wave / HW;
  int tile;
  const int s = find_tile(start_loc, n_seq, QW * 16, blockIdx.x, &tile);
  const int g = blockIdx.y, rep = a.H / G;
  const int hz = blockIdx.z * HW + hw;
  const int s0 = start_loc[s], s1 = start_loc[s + 1];
  const int bq0 = s0 + tile * QW * 16;
  if (bq0 >= s1) return;  // the whole block: no barrier is skipped
  const int bnq = min(QW * 16, s1 - bq0);
  const int bpos_min = positions[bq0], bpos_max = bpos_min + bnq - 1;
  const int q0 = bq0 + qw * 16;
  const bool wave_on = q0 < s1 && hz < rep;
  const int nq = wave_on ? min(16, s1 - q0) : 0;
  const int h = g * rep + min(hz, rep - 1);
  const bool q_ok = wave_on && col < nq;
  const int tq = wave_on ? q0 + min(col, nq - 1) : bq0;
  const int pos_q = q_ok ? positions[tq] : -1;
  const int wpos_min = wave_on ? positions[q0] : 0, wpos_max = wpos_min + nq - 1;
  const int lo_q = q_ok ? a.lower(pos_q) : 0;
  const int wlo = a.lower(wpos_min), wlo_max = a.lower(max(wpos_max, 0));
  const int blo = a.lower(bpos_min);
  // tiles of the kept first tokens, then from the first query's window on
  const int kept = a.kept(blo), n_kept = (kept + kKT - 1) / kKT;
  const int n_tiles = n_kept + (bpos_max - blo) / kKT + 1;
  const int* bt = block_tables + (size_t)s * max_blocks;
  const int nf = D / Frag::kDims, ndt = Dv / 16;
  const int krow = D + kRPad, vrow = kTied ? krow : Dv + kRPad;
  const int k_elems = kKT * krow, v_elems = kTied ? 0 : kKT * vrow;
  const int buf_elems = k_elems + v_elems + 2 * kKT;  // + key scales (fp32)
  const int kcpr = D / 8, vcpr = Dv / 8;  // 16-byte chunks per cached row
  const ScoreConsts consts(a, h);

  frag_t qf[kNF];
  const bf16raw* qrow = q + (size_t)tq * q_stride + h * D;
#pragma unroll
  for (int f = 0; f < kNF; ++f)
    if (kExact || f < nf) {
      const bf16raw* p = qrow + f * Frag::kDims + grp * Frag::kElems;
      if constexpr (kWideQK) {
        const bf16x4 x = *(const bf16x4*)p, y = *(const bf16x4*)(p + 4);
        qf[f] = (bf16x8){x[0], x[1], x[2], x[3], y[0], y[1], y[2], y[3]};
      } else {
        qf[f] = *(const bf16x4*)p;
      }
    }
  f32x4 oacc[kMaxDvTiles];
#pragma unroll
  for (int dt = 0; dt < kMaxDvTiles; ++dt) oacc[dt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;

  uint4 kreg[kKVec], vreg[kVVec];
  float kscr = 0.f;
  auto first_key = [&](int it) {
    return it < n_kept ? it * kKT : blo + (it - n_kept) * kKT;
  };
  auto last_key = [&](int it) { return it < n_kept ? kept - 1 : bpos_max; };
  auto cached_at = [&](int j, int64_t* blk, int* off) {
    *blk = bt[kExact ? j >> a.bs_shift : j / a.bs];
    *off = kExact ? j & (a.bs - 1) : j % a.bs;
  };
  auto load_tile = [&](int it) {
    const int j0 = first_key(it), j_end = last_key(it);
    int64_t blk;
    int off;
    if (a.kscale != nullptr && threadIdx.x < kKT) {
      cached_at(min(j0 + (int)threadIdx.x, j_end), &blk, &off);
      kscr = a.kscale[blk * a.bs + off];
    }
#pragma unroll
    for (int i = 0; i < kKVec; ++i) {
      const int v = i * nthr + threadIdx.x;
      const int row = v / kcpr, c = v % kcpr;
      if (row < kKT) {
        cached_at(min(j0 + row, j_end), &blk, &off);
        kreg[i] = *(const uint4*)(k_cache + ((blk * G + g) * a.bs + off) * D + c * 8);
      }
    }
    if constexpr (!kTied) {
#pragma unroll
      for (int i = 0; i < kVVec; ++i) {
        const int v = i * nthr + threadIdx.x;
        const int row = v / vcpr, c = v % vcpr;
        if (row < kKT) {
          cached_at(min(j0 + row, j_end), &blk, &off);
          vreg[i] = *(const uint4*)(v_cache +
              ((blk * (G / a.kvs) + g / a.kvs) * a.bs + off) * a.v_rs + c * 8);
        }
      }
    }
  };
  auto store_tile = [&](int buf) {
    bf16raw* ks_ = lds + buf * buf_elems;
#pragma unroll
    for (int i = 0; i < kKVec; ++i) {
      const int v = i * nthr + threadIdx.x;
      const int row = v / kcpr, c = v % kcpr;
      if (row < kKT) *(uint4*)(ks_ + row * krow + c * 8) = kreg[i];
    }
    if constexpr (!kTied) {
      bf16raw* vs_ = ks_ + k_elems;
#pragma unroll
      for (int i = 0; i < kVVec; ++i) {
        const int v = i * nthr + threadIdx.x;
        const int row = v / vcpr, c = v % vcpr;
        if (row < kKT) *(uint4*)(vs_ + row * vrow + c * 8) = vreg[i];
      }
    }
    if (a.kscale != nullptr && threadIdx.x < kKT)
      ((float*)(ks_ + k_elems + v_elems))[threadIdx.x] = kscr;
  };

  load_tile(0);
  store_tile(0);
  __syncthreads();
  int buf = 0;
  for (int it = 0; it < n_tiles; ++it, buf ^= 1) {
    const bool more = it + 1 < n_tiles;
    if (more) load_tile(it + 1);
    const int j0 = first_key(it);
    const bf16raw* ks_ = lds + buf * buf_elems;
    const bf16raw* vs_ = ks_ + (kTied ? 0 : k_elems);
    const float* kc_ = (const float*)(ks_ + k_elems + v_elems);
    // wave-uniform: something of this tile is visible to the wave's queries
    if (wave_on && j0 <= wpos_max && (j0 + kKT - 1 >= wlo || j0 < a.keep)) {
      f32x4 sacc[2];
      sacc[0] = sacc[1] = (f32x4){0.f, 0.f, 0.f, 0.f};
      const bf16raw* kp = ks_ + col * krow + grp * Frag::kElems;
#pragma unroll
      for (int f = 0; f < kNF; ++f)
        if (kExact || f < nf) {
          sacc[0] = mfma_qk(*(const frag_t*)(kp + f * Frag::kDims), qf[f], sacc[0]);
          sacc[1] = mfma_qk(*(const frag_t*)(kp + 16 * krow + f * Frag::kDims), qf[f],
                            sacc[1]);
        }
      // this lane: query `col`, keys j0 + sub * 16 + grp * 4 + i
      float sc[8];
      base2_scores<true>(sacc, consts, (float)(j0 + grp * 4 - pos_q),
                         a.kscale != nullptr ? kc_ + grp * 4 : nullptr, sc);
      // wave-uniform: a tile whose keys all queries see needs no mask. (Masks
      // are selects: hipcc 7.2 has lost such an assignment from under a branch.)
      const int jl = j0 + grp * 4;
      if (it < n_kept) {
        if (j0 + kKT > kept) {
#pragma unroll
          for (int e = 0; e < 8; ++e)
            sc[e] = jl + (e >> 2) * 16 + (e & 3) < kept ? sc[e] : -INFINITY;
        }
      } else if (nq < 16 || j0 + kKT - 1 > wpos_min || j0 < wlo_max) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int j = jl + (e >> 2) * 16 + (e & 3);
          const bool vis = (j <= pos_q) & ((j >= lo_q) | (j < a.keep));
          sc[e] = vis ? sc[e] : -INFINITY;
        }
      }
      float mt = sc[0];
#pragma unroll
      for (int e = 1; e < 8; ++e) mt = fmaxf(mt, sc[e]);
      mt = column_max(mt, lane);
      const float m_new = fmaxf(m, mt);
      // no visible key so far: keep everything at zero without forming inf - inf
      const float m_use = m_new == -INFINITY ? 0.f : m_new;
      const float corr = __builtin_amdgcn_exp2f(m - m_use);
      float pv[8];
      float ps = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        pv[e] = __builtin_amdgcn_exp2f(sc[e] - m_use);
        ps += pv[e];
      }
      union { bf16x8 v; uint32_t u[4]; } pk;
#pragma unroll
      for (int e = 0; e < 4; ++e) pk.u[e] = cvt_pk_bf16(pv[2 * e], pv[2 * e + 1]);
      const bf16x8 pb = pk.v;
      l = l * corr + ps;
      m = m_new;
      const bf16raw* vp = vs_ + (grp * 4 + (col >> 2)) * vrow + (col & 3) * 4;
#pragma unroll
      for (int dt = 0; dt < kMaxDvTiles; ++dt) {
        if (kExact || dt < ndt) {
          const bf16x4 v0 = lds_read_transposed(vp + dt * 16);
          const bf16x4 v1 = lds_read_transposed(vp + dt * 16 + 16 * vrow);
          const bf16x8 vf = (bf16x8){v0[0], v0[1], v0[2], v0[3], v1[0], v1[1], v1[2], v1[3]};
          f32x4 o = oacc[dt];
          o[0] *= corr; o[1] *= corr; o[2] *= corr; o[3] *= corr;
          oacc[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pb, o, 0, 0, 0);
        }
      }
    }
    if (more) store_tile(buf ^ 1);
    __syncthreads();
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  if (a.sink != nullptr) l += __builtin_amdgcn_exp2f(a.sink[h] * kLog2e - m);
  if (q_ok) {
    const float inv = a.out_factor<bf16raw>(tq, h) / l;
    bf16raw* op = out + (size_t)tq * out_stride + h * Dv + grp * 4;
#pragma unroll
    for (int dt = 0; dt < kMaxDvTiles; ++dt) {
      if (kExact || dt < ndt) {
        ushort4 o4;
        o4.x = f32_to_bf16(oacc[dt][0] * inv);
        o4.y = f32_to_bf16(oacc[dt][1] * inv);
        o4.z = f32_to_bf16(oacc[dt][2] * inv);
        o4.w = f32_to_bf16(oacc[dt][3] * inv);
        *(ushort4*)(op + dt * 16) = o4;
      }
    }
  }
}

}  // namespace

static bool dense_heads3(const torch::Tensor& t) {
  // heads are addressed as row + h * size(2): a single head's stride is free
  return t.dim() == 3 && (t.size(2) == 1 || t.stride(2) == 1) &&
         (t.size(1) == 1 || t.stride(1) == t.size(2));
}

void rope_pairs_and_cache(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                          torch::Tensor positions, torch::Tensor inv_freq,
                          torch::Tensor k_cache, torch::Tensor v_cache,
                          torch::Tensor slot_mapping) {
  check_i32(positions, "positions");
  check_f32(inv_freq, "inv_freq");
  TORCH_CHECK(dense_heads3(q) && dense_heads3(k) && dense_heads3(v));
  TORCH_CHECK(slot_mapping.scalar_type() == torch::kInt64 &&
              slot_mapping.is_contiguous());
  const int T = q.size(0), H = q.size(1), D = q.size(2);
  const int G = k.size(1), Dv = v.size(2), half = inv_freq.numel();
  TORCH_CHECK(D % 2 == 0 && 2 * half <= D, "key size must be even and hold the rotated dims");
  TORCH_CHECK(k.size(0) == T && v.size(0) == T && k.size(2) == D && v.size(1) == G);
  TORCH_CHECK(positions.numel() == T && slot_mapping.numel() == T);
  TORCH_CHECK(k_cache.is_contiguous() && v_cache.is_contiguous() &&
              k_cache.dim() == 4 && v_cache.dim() == 4);
  TORCH_CHECK(k_cache.size(1) == G && k_cache.size(3) == D && v_cache.size(1) == G &&
              v_cache.size(3) == Dv && v_cache.size(2) == k_cache.size(2) &&
              v_cache.size(0) == k_cache.size(0));
  TORCH_CHECK(k.scalar_type() == q.scalar_type() && v.scalar_type() == q.scalar_type() &&
              k_cache.scalar_type() == q.scalar_type() &&
              v_cache.scalar_type() == q.scalar_type());
  if (T == 0) return;
  SEQ_DISPATCH_ACT(q, {
    hipLaunchKernelGGL((rope_pairs_cache_kernel<act_t>), dim3(T), dim3(256), 0,
                       SEQ_STREAM(), (act_t*)q.data_ptr(), q.stride(0),
                       (const act_t*)k.data_ptr(), k.stride(0),
                       (const act_t*)v.data_ptr(), v.stride(0),
                       (const int*)positions.data_ptr(),
                       (const float*)inv_freq.data_ptr(), half,
                       (act_t*)k_cache.data_ptr(), (act_t*)v_cache.data_ptr(),
                       (const int64_t*)slot_mapping.data_ptr(), H, G, D, Dv,
                       (int)k_cache.size(2));
  });
  SEQ_CHECK_LAUNCH();
}

void qknorm_rope_half_and_cache(torch::Tensor q, torch::Tensor k, torch::Tensor v,
                                c10::optional<torch::Tensor> q_weight,
                                c10::optional<torch::Tensor> k_weight, double eps,
                                torch::Tensor positions, torch::Tensor inv_freq,
                                torch::Tensor k_cache, torch::Tensor v_cache,
                                torch::Tensor slot_mapping) {
  check_i32(positions, "positions");
  check_f32(inv_freq, "inv_freq");
  TORCH_CHECK(dense_heads3(q) && dense_heads3(k) && dense_heads3(v));
  TORCH_CHECK(slot_mapping.scalar_type() == torch::kInt64 &&
              slot_mapping.is_contiguous());
  const int T = q.size(0), H = q.size(1), D = q.size(2);
  const int G = k.size(1), Dv = v.size(2), half = inv_freq.numel();
  TORCH_CHECK(2 * half <= D, "rotated dims exceed the key size");
  TORCH_CHECK(k.size(0) == T && v.size(0) == T && k.size(2) == D && v.size(1) == G);
  TORCH_CHECK(positions.numel() == T && slot_mapping.numel() == T);
  TORCH_CHECK(q_weight.has_value() == k_weight.has_value());
  if (q_weight.has_value()) {
    check_f32(*q_weight, "q_weight");
    check_f32(*k_weight, "k_weight");
    TORCH_CHECK(q_weight->numel() == (int64_t)H * D && k_weight->numel() == (int64_t)G * D);
  }
  TORCH_CHECK(k_cache.is_contiguous() && v_cache.is_contiguous() &&
              k_cache.dim() == 4 && v_cache.dim() == 4);
  TORCH_CHECK(k_cache.size(1) == G && k_cache.size(3) == D && v_cache.size(1) == G &&
              v_cache.size(3) == Dv && v_cache.size(2) == k_cache.size(2) &&
              v_cache.size(0) == k_cache.size(0));
  TORCH_CHECK(k.scalar_type() == q.scalar_type() && v.scalar_type() == q.scalar_type() &&
              k_cache.scalar_type() == q.scalar_type() &&
              v_cache.scalar_type() == q.scalar_type());
  if (T == 0) return;
  SEQ_DISPATCH_ACT(q, {
    hipLaunchKernelGGL((qknorm_rope_half_cache_kernel<act_t>), dim3(T), dim3(256), 0,
                       SEQ_STREAM(), (act_t*)q.data_ptr(), q.stride(0),
                       (const act_t*)k.data_ptr(), k.stride(0),
                       (const act_t*)v.data_ptr(), v.stride(0),
                       q_weight.has_value() ? (const float*)q_weight->data_ptr() : nullptr,
                       k_weight.has_value() ? (const float*)k_weight->data_ptr() : nullptr,
                       (float)eps, (const int*)positions.data_ptr(),
                       (const float*)inv_freq.data_ptr(), half,
                       (act_t*)k_cache.data_ptr(), (act_t*)v_cache.data_ptr(),
                       (const int64_t*)slot_mapping.data_ptr(), H, G, D, Dv,
                       (int)k_cache.size(2));
  });
  SEQ_CHECK_LAUNCH();
}

void headnorm_qk_to_cache(torch::Tensor q, torch::Tensor k, torch::Tensor v, double eps,
                          torch::Tensor k_cache, torch::Tensor v_cache,
                          torch::Tensor slot_mapping) {
  TORCH_CHECK(q.is_cuda() && k.is_cuda() && v.is_cuda() && dense_heads3(q) &&
              dense_heads3(k) && dense_heads3(v));
  TORCH_CHECK(slot_mapping.scalar_type() == torch::kInt64 &&
              slot_mapping.is_contiguous() && slot_mapping.is_cuda());
  const int T = q.size(0), H = q.size(1), D = q.size(2), G = k.size(1), Dv = v.size(2);
  TORCH_CHECK(k.size(0) == T && v.size(0) == T && k.size(2) == D && v.size(1) == G &&
              slot_mapping.numel() == T);
  TORCH_CHECK(k_cache.is_cuda() && v_cache.is_cuda() && k_cache.is_contiguous() &&
              v_cache.is_contiguous() && k_cache.dim() == 4 && v_cache.dim() == 4);
  TORCH_CHECK(k_cache.size(1) == G && k_cache.size(3) == D && v_cache.size(1) == G &&
              v_cache.size(3) == Dv && v_cache.size(2) == k_cache.size(2) &&
              v_cache.size(0) == k_cache.size(0));
  TORCH_CHECK(k.scalar_type() == q.scalar_type() && v.scalar_type() == q.scalar_type() &&
              k_cache.scalar_type() == q.scalar_type() &&
              v_cache.scalar_type() == q.scalar_type());
  if (T == 0) return;
  const int n = 16 / q.element_size();
  auto al = [&](const torch::Tensor& x) {
    return ((size_t)x.data_ptr()) % 16 == 0 && x.stride(0) % n == 0;
  };
  int lpr = 1;
  while (lpr * n < D) lpr *= 2;
  const bool vec = D % n == 0 && Dv % n == 0 && lpr <= WAVE && al(q) && al(k) && al(v) &&
                   ((size_t)k_cache.data_ptr()) % 16 == 0 &&
                   ((size_t)v_cache.data_ptr()) % 16 == 0;
  SEQ_DISPATCH_ACT(q, {
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(T), dim3(256), 0, SEQ_STREAM(), (act_t*)q.data_ptr(),
                         q.stride(0), (const act_t*)k.data_ptr(), k.stride(0),
                         (const act_t*)v.data_ptr(), v.stride(0), (float)eps,
                         (act_t*)k_cache.data_ptr(), (act_t*)v_cache.data_ptr(),
                         (const int64_t*)slot_mapping.data_ptr(), H, G, D, Dv,
                         (int)k_cache.size(2), lpr);
    };
    if (vec) launch(headnorm_qk_cache_kernel<act_t, true>);
    else launch(headnorm_qk_cache_kernel<act_t, false>);
  });
  SEQ_CHECK_LAUNCH();
}

void qnorm_rows_to_cache(torch::Tensor q, torch::Tensor k, torch::Tensor q_weight,
                         double eps, torch::Tensor cache, torch::Tensor key_scale,
                         torch::Tensor slot_mapping) {
  check_f32(q_weight, "q_weight");
  check_f32(key_scale, "key_scale");
  TORCH_CHECK(q.dim() == 3 && k.dim() == 3 && dense_heads3(q) && dense_heads3(k));
  TORCH_CHECK(slot_mapping.scalar_type() == torch::kInt64 &&
              slot_mapping.is_contiguous() && slot_mapping.is_cuda());
  const int T = q.size(0), H = q.size(1), D = q.size(2), G = k.size(1);
  TORCH_CHECK(k.size(0) == T && k.size(2) == D && slot_mapping.numel() == T &&
              q_weight.numel() == (int64_t)H * D);
  TORCH_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.dim() == 4 &&
              cache.size(1) == G && cache.size(3) == D &&
              key_scale.numel() == cache.size(0) * cache.size(2));
  TORCH_CHECK(k.scalar_type() == q.scalar_type() && cache.scalar_type() == q.scalar_type());
  if (T == 0) return;
  const int n = 16 / q.element_size();
  auto al = [&](const torch::Tensor& x) {
    return ((size_t)x.data_ptr()) % 16 == 0 && x.stride(0) % n == 0;
  };
  const bool vec = D % n == 0 && al(q) && al(k) && ((size_t)cache.data_ptr()) % 16 == 0;
  SEQ_DISPATCH_ACT(q, {
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(T), dim3(256), 0, SEQ_STREAM(), (act_t*)q.data_ptr(),
                         q.stride(0), (const act_t*)k.data_ptr(), k.stride(0),
                         (const float*)q_weight.data_ptr(), (float)eps,
                         (act_t*)cache.data_ptr(), (float*)key_scale.data_ptr(),
                         (const int64_t*)slot_mapping.data_ptr(), H, G, D,
                         (int)cache.size(2));
    };
    if (vec) launch(qnorm_rows_cache_kernel<act_t, true>);
    else launch(qnorm_rows_cache_kernel<act_t, false>);
  });
  SEQ_CHECK_LAUNCH();
}

void masked_paged_attention(torch::Tensor out, torch::Tensor q,
                            torch::Tensor k_cache, torch::Tensor v_cache,
                            torch::Tensor block_tables, torch::Tensor start_loc,
                            torch::Tensor token_seq, torch::Tensor positions,
                            int64_t max_len, double scale, double softcap,
                            int64_t chunk, int64_t window, double out_scale,
                            c10::optional<torch::Tensor> sink_scores,
                            int64_t keep_first, c10::optional<torch::Tensor> slopes,
                            c10::optional<torch::Tensor> key_scale,
                            c10::optional<torch::Tensor> head_gate) {
  check_i32(start_loc, "start_loc");
  check_i32(block_tables, "block_tables");
  check_i32(token_seq, "token_seq");
  check_i32(positions, "positions");
  TORCH_CHECK(dense_heads3(q) && dense_heads3(out));
  const int T = q.size(0), H = q.size(1), D = q.size(2);
  TORCH_CHECK(k_cache.is_contiguous() && k_cache.dim() == 4 && v_cache.dim() == 4);
  const int G = k_cache.size(1), bs = k_cache.size(2), Dv = v_cache.size(3);
  // the value cache may have fewer heads than the key cache: kvs key heads
  // (score maps over the same values) share one value head
  const int Gv = v_cache.size(1);
  TORCH_CHECK(k_cache.size(3) == D && Gv > 0 && G % Gv == 0 && v_cache.size(2) == bs);
  const int kvs = G / Gv;
  // value rows may be the leading columns of wider rows (of the key rows,
  // when a layer caches one row per token that serves as both)
  const int64_t v_rs = v_cache.stride(2);
  TORCH_CHECK(v_cache.is_cuda() && (Dv == 1 || v_cache.stride(3) == 1) && v_rs >= Dv &&
              v_cache.stride(1) == (int64_t)bs * v_rs &&
              v_cache.stride(0) == (int64_t)Gv * bs * v_rs,
              "value cache rows must be evenly spaced");
  AttnArgs args{};
  if (sink_scores.has_value()) {
    check_f32(*sink_scores, "sink_scores");
    TORCH_CHECK(sink_scores->numel() == H, "one sink score per head");
    args.sink = (const float*)sink_scores->data_ptr();
  }
  if (slopes.has_value()) {
    check_f32(*slopes, "slopes");
    TORCH_CHECK(slopes->numel() == H, "one slope per head");
    args.slopes = (const float*)slopes->data_ptr();
  }
  if (key_scale.has_value()) {
    check_f32(*key_scale, "key_scale");
    TORCH_CHECK(key_scale->numel() == k_cache.size(0) * bs, "one scale per cached key");
    args.kscale = (const float*)key_scale->data_ptr();
  }
  if (head_gate.has_value()) {
    check_rows(*head_gate, "head_gate");
    TORCH_CHECK(head_gate->size(0) == T && head_gate->size(1) == H &&
                head_gate->scalar_type() == q.scalar_type(),
                "one gate per token and head, of q's dtype");
    args.gate = head_gate->data_ptr();
    args.gate_rs = head_gate->stride(0);
  }
  TORCH_CHECK(keep_first >= 0 && (keep_first == 0 || (chunk == 0 && window > 0)),
              "kept first tokens belong to a window");
  args.scale = (float)scale;
  args.softcap = (float)softcap;
  args.out_scale = (float)out_scale;
  args.chunk = (int)chunk;
  args.window = (int)window;
  args.keep = (int)keep_first;
  args.v_rs = v_rs;
  args.H = H; args.G = G; args.D = D; args.Dv = Dv; args.bs = bs; args.kvs = kvs;
  args.bs_shift = -1;
  for (int i = 0; i < 20; ++i)
    if (bs == 1 << i) args.bs_shift = i;
  // one row per token and head that is key and (its leading part) value
  const bool tied = v_cache.data_ptr() == k_cache.data_ptr() && kvs == 1 && v_rs == D &&
                    Dv <= D;
  TORCH_CHECK(G > 0 && H % G == 0 && H <= 65535);
  TORCH_CHECK(out.size(0) == T && out.size(1) == H && out.size(2) == Dv);
  TORCH_CHECK(Dv <= kMaxDvPerLane * WAVE, "value size too large");
  TORCH_CHECK(block_tables.dim() == 2 && token_seq.numel() == T &&
              positions.numel() == T);
  TORCH_CHECK(k_cache.scalar_type() == q.scalar_type() &&
              v_cache.scalar_type() == q.scalar_type() &&
              out.scalar_type() == q.scalar_type());
  if (T == 0) return;
  const int n_seq = start_loc.numel() - 1;
  TORCH_CHECK(block_tables.size(0) >= n_seq);
  auto al8 = [](const torch::Tensor& t) {
    return ((size_t)t.data_ptr()) % 8 == 0 && t.stride(0) % 4 == 0;
  };
  if (q.scalar_type() == torch::kBFloat16 && max_len > 1 && D % 16 == 0 &&
      Dv % 16 == 0 && D <= 512 && Dv <= 512 && al8(q) && al8(out) && v_rs % 8 == 0) {
    // prompt portions: matrix-core kernel over 16-query tiles of every run
    const int tiles = T / 16 + n_seq;
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(tiles, H), dim3(WAVE), 0, SEQ_STREAM(),
                         (bf16raw*)out.data_ptr(), out.stride(0),
                         (const bf16raw*)q.data_ptr(), q.stride(0),
                         (const bf16raw*)k_cache.data_ptr(),
                         (const bf16raw*)v_cache.data_ptr(),
                         (const int*)block_tables.data_ptr(),
                         (int)block_tables.size(1), (const int*)start_loc.data_ptr(),
                         (const int*)positions.data_ptr(), n_seq, args);
    };
    const size_t lds_shared =
        (size_t)2 * (kKT * (D + kRPad) + (tied ? 0 : kKT * (Dv + kRPad)) + 2 * kKT) *
        sizeof(bf16raw);
    const bool cache_al16 = ((size_t)k_cache.data_ptr()) % 16 == 0 &&
                            ((size_t)v_cache.data_ptr()) % 16 == 0;
    if (D <= 256 && Dv <= 256 && lds_shared <= 64 * 1024 && cache_al16) {
      // tiles shared through LDS by up to 8 waves: heads of a group first,
      // then neighbouring query tiles
      const int rep = H / G;
      int HW = 1;
      while (HW * 2 <= rep && HW < 8) HW *= 2;
      constexpr int WPB = kPrefillThreads / WAVE;
      const int QW = WPB / HW;
      const int btiles = T / (QW * 16) + n_seq;
      const int zb = (rep + HW - 1) / HW;
      TORCH_CHECK(G <= 65535 && zb <= 65535);
      auto launch_shared = [&](auto kern) {
      hipLaunchKernelGGL(kern,
                         dim3(btiles, G, zb), dim3(WPB * WAVE), lds_shared,
                         SEQ_STREAM(), (bf16raw*)out.data_ptr(), out.stride(0),
                         (const bf16raw*)q.data_ptr(), q.stride(0),
                         (const bf16raw*)k_cache.data_ptr(),
                         (const bf16raw*)v_cache.data_ptr(),
                         (const int*)block_tables.data_ptr(),
                         (int)block_tables.size(1), (const int*)start_loc.data_ptr(),
                         (const int*)positions.data_ptr(), n_seq, HW, QW, args);
      };
      auto sized = [&](auto is_tied) {
        constexpr bool kT = decltype(is_tied)::value;
        const bool shift = args.bs_shift >= 0, wide = D % 32 == 0;
        if (shift && D == 128 && Dv == 128)
          launch_shared(masked_prefill_mfma_shared_kernel<8, 8, true, kT, true>);
        else if (shift && D == 64 && Dv == 64)
          launch_shared(masked_prefill_mfma_shared_kernel<4, 4, true, kT, true>);
        else if (shift && !kT && D == 64 && Dv == 128)
          launch_shared(masked_prefill_mfma_shared_kernel<4, 8, true, false, true>);
        else if (shift && kT && D == 192 && Dv == 128)
          launch_shared(masked_prefill_mfma_shared_kernel<12, 8, true, true, true>);
        else if (D <= 128 && Dv <= 128 && wide)
          launch_shared(masked_prefill_mfma_shared_kernel<8, 8, true, kT, false>);
        else if (D <= 128 && Dv <= 128)
          launch_shared(masked_prefill_mfma_shared_kernel<8, 8, false, kT, false>);
        // larger keys (a latent with a rotated part behind it) or values keep
        // more fragments in registers
        else if (D <= 128 && wide)
          launch_shared(masked_prefill_mfma_shared_kernel<8, 16, true, kT, false>);
        else if (wide)
          launch_shared(masked_prefill_mfma_shared_kernel<16, 16, true, kT, false>);
        else
          launch_shared(masked_prefill_mfma_shared_kernel<16, 16, false, kT, false>);
      };
      if (tied) sized(std::true_type{});
      else sized(std::false_type{});
    } else if (D <= 128 && Dv <= 256) {
      launch(masked_prefill_mfma_kernel<8, 16>);
    } else {
      launch(masked_prefill_mfma_kernel<32, 32>);
    }
    SEQ_CHECK_LAUNCH();
    return;
  }
  if (q.scalar_type() == torch::kBFloat16 && max_len == 1 && al8(q) &&
      masked_decode_mfma(out, q, k_cache, v_cache, block_tables, token_seq, positions, args,
                         tied))
    return;
  SEQ_DISPATCH_ACT(q, {
    constexpr int N = Vec16<act_t>::N;
    // 16-byte row loads need whole vectors per key / value row and at most
    // one wave of lanes per value row
    const bool vec = D % N == 0 && Dv % N == 0 && Dv / N <= WAVE && Dv >= N &&
                     N <= kMaxDvPerLane && v_rs % N == 0 &&
                     ((size_t)v_cache.data_ptr()) % 16 == 0;
    const int ngrp = vec ? WAVE / (Dv / N) : 1;
    const size_t lds = (size_t)(3 * WAVE * kDecWaves + 2 * kDecWaves +
                                ((D + 3) & ~3) + kDecWaves * ngrp * Dv) * 4;
    TORCH_CHECK(lds <= 64 * 1024, "attention scratch exceeds LDS");
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(T, H), dim3(kDecWaves * WAVE), lds, SEQ_STREAM(),
                         (act_t*)out.data_ptr(), out.stride(0),
                         (const act_t*)q.data_ptr(), q.stride(0),
                         (const act_t*)k_cache.data_ptr(),
                         (const act_t*)v_cache.data_ptr(),
                         (const int*)block_tables.data_ptr(),
                         (int)block_tables.size(1), (const int*)token_seq.data_ptr(),
                         (const int*)positions.data_ptr(), args);
    };
    if (vec) launch(masked_paged_attention_kernel<act_t, true>);
    else launch(masked_paged_attention_kernel<act_t, false>);
  });
  SEQ_CHECK_LAUNCH();
}
