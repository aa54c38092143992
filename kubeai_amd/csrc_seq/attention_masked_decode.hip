// Single decode tokens of masked attention on the matrix cores (bf16).
#include "attn_masked.h"

#include <algorithm>
#include <type_traits>

namespace {

constexpr int kDW = 4;  // waves of a decode block; each takes every fourth key tile

// decode blocks a CU holds (waves per SIMD); a tile is a chain of dependent
// steps, so other waves have to fill its gaps
constexpr int decode_blocks_per_cu(int d_steps, bool tied) {
  return d_steps > 8 ? 2 : tied ? 4 : 3;
}

// bytes of a wave's staging region: a 32-row value tile + key scales
inline __host__ __device__ int decode_stage_bytes(int Dv) {
  return kKT * (Dv + kRPad) * (int)sizeof(bf16raw) + kKT * (int)sizeof(float);
}

// grid (T, G, ceil(rep / 16) * splits): the 16 rows of an MFMA tile are the
// query heads that share one key/value head (all heads of a latent layer, the
// group of a grouped layer), so a key or value row is loaded once for all of
// them. The visible keys are numbered through (kept first tokens, then the
// window) and cut into 32-key tiles; the four waves walk disjoint tiles. A
// lane loads its pieces of two rows per tile straight as MFMA operands, one
// tile ahead; the value part (kTied: the same registers) is written to a
// wave-private LDS tile and comes back through the transposing LDS read.
// Statistics are fp32 in the base-2 domain, and the waves' partial results are
// joined through LDS. kExact: the sizes are D = 16 kMaxDSteps, Dv = 16
// kMaxDvTiles and the block size is a power of two; otherwise the template
// sizes are bounds, and every step is guarded (and so waits for itself).
template <int kMaxDSteps, int kMaxDvTiles, bool kWide, bool kTied, bool kExact>
__global__ __launch_bounds__(kDW * WAVE, decode_blocks_per_cu(kMaxDSteps, kTied))
void masked_decode_mfma_kernel(
    bf16raw* __restrict__ out, int64_t out_stride, const bf16raw* __restrict__ q,
    int64_t q_stride, const bf16raw* __restrict__ k_cache,
    const bf16raw* __restrict__ v_cache, const int* __restrict__ block_tables,
    int max_blocks, const int* __restrict__ token_seq,
    const int* __restrict__ positions, int n_split, float* __restrict__ part_o,
    float* __restrict__ part_ml, AttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  typedef QkFrag<kWide> Frag;
  typedef typename Frag::type frag_t;
  constexpr int kNF = kMaxDSteps * 16 / Frag::kDims;
  constexpr int kNV = kMaxDvTiles * 16 / Frag::kDims;
  const int H = a.H, G = a.G;
  const int D = kExact ? kMaxDSteps * 16 : a.D, Dv = kExact ? kMaxDvTiles * 16 : a.Dv;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int col = lane & 15, grp = lane >> 4;
  const int t = blockIdx.x, g = blockIdx.y, rep = H / G;
  const int zt = blockIdx.z / n_split, sp = blockIdx.z % n_split;
  const int h0 = g * rep + zt * 16;
  const int nh = min(16, (g + 1) * rep - h0);
  const int pos = positions[t];
  const int* bt = block_tables + (size_t)token_seq[t] * max_blocks;
  const int lo = a.lower(pos), kept = a.kept(lo), n_keys = kept + pos - lo + 1;
  const int nf = D / Frag::kDims, nv = Dv / Frag::kDims, ndt = Dv / 16;
  const int vrow = Dv + kRPad;
  bf16raw* vt = (bf16raw*)(smem + (size_t)wave * decode_stage_bytes(Dv));
  float* kc = (float*)(vt + kKT * vrow);
  const int hq = h0 + min(col, nh - 1);
  const bool scaled = a.kscale != nullptr, biased = a.slopes != nullptr;
  // the tiles dealt to the splits in contiguous shares
  const int n_tiles = (n_keys + kKT - 1) / kKT;
  const int per_split = (n_tiles + n_split - 1) / n_split;
  const int tile_end = min(n_tiles, (sp + 1) * per_split);
  int jn[2], bn[2];  // the lane's two keys of the tile to load, and their blocks
  frag_t kf[2][kNF], vf[2][kTied ? 1 : kNV];
  float ksr[2] = {1.f, 1.f};
  auto find_rows = [&](int tile) {
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) {
      const int v = min(tile * kKT + sub * 16 + col, n_keys - 1);
      jn[sub] = v < kept ? v : lo + v - kept;
      bn[sub] = bt[kExact ? jn[sub] >> a.bs_shift : jn[sub] / a.bs];
    }
  };
  auto load_rows = [&]() {
    int64_t krow_at[2], vrow_at[2];
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) {
      const int off = kExact ? jn[sub] & (a.bs - 1) : jn[sub] % a.bs;
      krow_at[sub] = (((int64_t)bn[sub] * G + g) * a.bs + off) * D;
      vrow_at[sub] = (((int64_t)bn[sub] * (G / a.kvs) + g / a.kvs) * a.bs + off) * a.v_rs;
      if (scaled) ksr[sub] = a.kscale[(int64_t)bn[sub] * a.bs + off];
    }
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) {
      const bf16raw* kp = k_cache + krow_at[sub] + grp * Frag::kElems;
#pragma unroll
      for (int f = 0; f < kNF; ++f)
        if (kExact || f < nf) kf[sub][f] = *(const frag_t*)(kp + f * Frag::kDims);
      if constexpr (!kTied) {
        const bf16raw* vp = v_cache + vrow_at[sub] + grp * Frag::kElems;
#pragma unroll
        for (int f = 0; f < kNV; ++f)
          if (kExact || f < nv) vf[sub][f] = *(const frag_t*)(vp + f * Frag::kDims);
      }
    }
  };
  int tile = sp * per_split + wave;
  if (tile < tile_end) {
    find_rows(tile);
    load_rows();
    if (tile + kDW < tile_end) find_rows(tile + kDW);
  }
  const ScoreConsts consts(a, hq);
  frag_t qf[kNF];
#pragma unroll
  for (int f = 0; f < kNF; ++f)
    if (kExact || f < nf) {
      const bf16raw* p =
          q + (size_t)t * q_stride + (size_t)hq * D + f * Frag::kDims + grp * Frag::kElems;
      if constexpr (kWide) {
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
  for (; tile < tile_end; tile += kDW) {
    f32x4 sacc[2];
    if (grp == 0) {
      kc[col] = ksr[0];
      kc[16 + col] = ksr[1];
    }
#pragma unroll
    for (int sub = 0; sub < 2; ++sub) {
      bf16raw* vw = vt + (sub * 16 + col) * vrow + grp * Frag::kElems;
#pragma unroll
      for (int f = 0; f < kNV; ++f)
        if (kExact || f < nv)
          *(frag_t*)(vw + f * Frag::kDims) = kTied ? kf[sub][f] : vf[sub][kTied ? 0 : f];
      sacc[sub] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int f = 0; f < kNF; ++f)
      if (kExact || f < nf) {
        sacc[0] = mfma_qk(kf[0][f], qf[f], sacc[0]);
        sacc[1] = mfma_qk(kf[1][f], qf[f], sacc[1]);
      }
    if (tile + kDW < tile_end) {
      load_rows();
      if (tile + 2 * kDW < tile_end) find_rows(tile + 2 * kDW);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    // this lane: head `col`, keys v0 + sub * 16 + grp * 4 + i of the numbering
    const int v0 = tile * kKT;
    float sc[8];
    base2_scores<false>(sacc, consts, 0.f, scaled ? kc + grp * 4 : nullptr, sc);
    if (biased) {
      if (v0 < kept) {  // kept first tokens and what follows them
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int v = v0 + (e >> 2) * 16 + grp * 4 + (e & 3);
          sc[e] += consts.slope2 * (float)((v < kept ? v : lo + v - kept) - pos);
        }
      } else {
        const float b = consts.slope2 * (float)(lo - kept - pos + v0 + grp * 4);
#pragma unroll
        for (int e = 0; e < 8; ++e)
          sc[e] += fmaf(consts.slope2, (float)((e >> 2) * 16 + (e & 3)), b);
      }
    }
    if (v0 + kKT > n_keys) {
#pragma unroll
      for (int e = 0; e < 8; ++e)
        sc[e] = v0 + (e >> 2) * 16 + grp * 4 + (e & 3) < n_keys ? sc[e] : -INFINITY;
    }
    float mt = sc[0];
#pragma unroll
    for (int e = 1; e < 8; ++e) mt = fmaxf(mt, sc[e]);
    mt = column_max(mt, lane);
    const float m_new = fmaxf(m, mt);  // finite: the tile's first key is visible
    const float corr = __builtin_amdgcn_exp2f(m - m_new);
    float pv[8];
    float ps = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      pv[e] = __builtin_amdgcn_exp2f(sc[e] - m_new);
      ps += pv[e];
    }
    union { bf16x8 v; uint32_t u[4]; } pk;
#pragma unroll
    for (int e = 0; e < 4; ++e) pk.u[e] = cvt_pk_bf16(pv[2 * e], pv[2 * e + 1]);
    l = l * corr + ps;
    m = m_new;
    const bf16raw* vp = vt + (grp * 4 + (col >> 2)) * vrow + (col & 3) * 4;
#pragma unroll
    for (int dt = 0; dt < kMaxDvTiles; ++dt) {
      if (kExact || dt < ndt) {
        const bf16x4 v0t = lds_read_transposed(vp + dt * 16);
        const bf16x4 v1t = lds_read_transposed(vp + dt * 16 + 16 * vrow);
        const bf16x8 vfr = (bf16x8){v0t[0], v0t[1], v0t[2], v0t[3],
                                    v1t[0], v1t[1], v1t[2], v1t[3]};
        f32x4 o = oacc[dt];
        o[0] *= corr; o[1] *= corr; o[2] *= corr; o[3] *= corr;
        oacc[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vfr, pk.v, o, 0, 0, 0);
      }
    }
    // all lanes read the tile before it is rewritten
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  __syncthreads();  // the staging regions are reused for the join
  float* cm = (float*)smem;            // [waves][16] running max (base 2)
  float* cl = cm + kDW * 16;           // [waves][16] sums
  float* co = cl + kDW * 16;           // [waves][16][Dv] unnormalised outputs
  if (grp == 0) {
    cm[wave * 16 + col] = m;
    cl[wave * 16 + col] = l;
  }
  if (col < nh) {
#pragma unroll
    for (int dt = 0; dt < kMaxDvTiles; ++dt)
      if (kExact || dt < ndt)
        *(f32x4*)(co + ((size_t)wave * 16 + col) * Dv + dt * 16 + grp * 4) = oacc[dt];
  }
  __syncthreads();
  for (int idx = threadIdx.x; idx < nh * Dv; idx += blockDim.x) {
    const int hh = idx / Dv, d = idx % Dv;
    float mx = -INFINITY;
#pragma unroll
    for (int w = 0; w < kDW; ++w) mx = fmaxf(mx, cm[w * 16 + hh]);
    float lsum = 0.f, x = 0.f;
#pragma unroll
    for (int w = 0; w < kDW; ++w) {
      const float mw = cm[w * 16 + hh];
      const float wsc = mw == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mw - mx);
      lsum += cl[w * 16 + hh] * wsc;
      x += co[((size_t)w * 16 + hh) * Dv + d] * wsc;
    }
    if (n_split == 1) {
      if (a.sink != nullptr) lsum += __builtin_amdgcn_exp2f(a.sink[h0 + hh] * kLog2e - mx);
      stf(out + (size_t)t * out_stride + (h0 + hh) * Dv + d,
          x * a.out_factor<bf16raw>(t, h0 + hh) / lsum);
    } else {
      // partial result of this split: [t][head][split] -> (max, sum), values
      const size_t row = ((size_t)t * H + h0 + hh) * n_split + sp;
      part_o[row * Dv + d] = x;
      if (d == 0) {
        part_ml[row * 2] = mx;
        part_ml[row * 2 + 1] = lsum;
      }
    }
  }
}

// Join of the key splits of masked_decode_mfma_kernel: grid (T, H), one wave;
// n_split <= 32. A lane holds one split's weight; splits without keys weigh 0.
__global__ __launch_bounds__(WAVE) void decode_split_join_kernel(
    bf16raw* __restrict__ out, int64_t out_stride, const float* __restrict__ part_o,
    const float* __restrict__ part_ml, int n_split, AttnArgs a) {
  const int H = a.H, Dv = a.Dv;
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const size_t row0 = ((size_t)t * H + h) * n_split;
  float2 ml = make_float2(-INFINITY, 0.f);
  if (lane < n_split) ml = *(const float2*)(part_ml + (row0 + lane) * 2);
  const float mx = wave_max(ml.x);
  const float w = __builtin_amdgcn_exp2f(ml.x - mx);
  float lsum = wave_sum(ml.y * w);
  if (a.sink != nullptr) lsum += __builtin_amdgcn_exp2f(a.sink[h] * kLog2e - mx);
  const float inv = a.out_factor<bf16raw>(t, h) / lsum;
  for (int d = lane; d < Dv; d += WAVE) {
    float x = 0.f;
#pragma unroll 4
    for (int s = 0; s < n_split; ++s)
      x += part_o[(row0 + s) * Dv + d] *
           __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, w), s));
    stf(out + (size_t)t * out_stride + h * Dv + d, x * inv);
  }
}

}  // namespace

bool masked_decode_mfma(const torch::Tensor& out, const torch::Tensor& q,
                        const torch::Tensor& k_cache, const torch::Tensor& v_cache,
                        const torch::Tensor& block_tables, const torch::Tensor& token_seq,
                        const torch::Tensor& positions, const AttnArgs& args, bool tied) {
  const int T = q.size(0), H = args.H, G = args.G, D = args.D, Dv = args.Dv;
  // worth it when several heads share a key row
  if (H / G < 4 || D % 16 != 0 || Dv % 16 != 0 || D > 256 || Dv > 128 ||
      args.v_rs % 8 != 0 || ((size_t)k_cache.data_ptr()) % 16 != 0 ||
      ((size_t)v_cache.data_ptr()) % 16 != 0)
    return false;
  const int rep = H / G, zb = (rep + 15) / 16;
  const size_t stage = (size_t)kDW * decode_stage_bytes(Dv);
  const size_t join = (size_t)kDW * (32 + 16 * Dv) * sizeof(float);
  // keys split over blocks until there is a block for every CU (past that, more
  // splits cost more in joins than shorter walks save), as long as every wave
  // has a tile at the longest context the block tables can describe; splits
  // beyond a sequence's keys exit at once
  int64_t cap = (int64_t)block_tables.size(1) * args.bs;
  if (args.window > 0) cap = std::min<int64_t>(cap, args.window + args.keep);
  if (args.chunk > 0) cap = std::min<int64_t>(cap, args.chunk);
  const int64_t room = 256 / ((int64_t)T * G * zb);
  int n_split = (int)std::max<int64_t>(
      1, std::min({room, (cap + kKT * kDW - 1) / (kKT * kDW), (int64_t)32}));
  TORCH_CHECK(G <= 65535 && (int64_t)zb * n_split <= 65535 && H <= 65535);
  torch::Tensor part_o, part_ml;
  if (n_split > 1) {
    auto f32 = torch::TensorOptions().dtype(torch::kFloat32).device(q.device());
    part_o = torch::empty({(int64_t)T * H * n_split, Dv}, f32);
    part_ml = torch::empty({(int64_t)T * H * n_split, 2}, f32);
  }
  auto launch = [&](auto kern) {
    hipLaunchKernelGGL(kern, dim3(T, G, zb * n_split), dim3(kDW * WAVE),
                       stage > join ? stage : join, SEQ_STREAM(), (bf16raw*)out.data_ptr(),
                       out.stride(0), (const bf16raw*)q.data_ptr(), q.stride(0),
                       (const bf16raw*)k_cache.data_ptr(),
                       (const bf16raw*)v_cache.data_ptr(),
                       (const int*)block_tables.data_ptr(), (int)block_tables.size(1),
                       (const int*)token_seq.data_ptr(), (const int*)positions.data_ptr(),
                       n_split, n_split > 1 ? (float*)part_o.data_ptr() : nullptr,
                       n_split > 1 ? (float*)part_ml.data_ptr() : nullptr, args);
  };
  auto sized = [&](auto is_tied) {
    constexpr bool kT = decltype(is_tied)::value;
    const bool shift = args.bs_shift >= 0;
    if (shift && D == 128 && Dv == 128) launch(masked_decode_mfma_kernel<8, 8, true, kT, true>);
    else if (shift && D == 64 && Dv == 64) launch(masked_decode_mfma_kernel<4, 4, true, kT, true>);
    else if (shift && !kT && D == 64 && Dv == 128)
      launch(masked_decode_mfma_kernel<4, 8, true, false, true>);
    else if (shift && kT && D == 192 && Dv == 128)
      launch(masked_decode_mfma_kernel<12, 8, true, true, true>);
    else if (D % 32 == 0 && Dv % 32 == 0 && D <= 128)
      launch(masked_decode_mfma_kernel<8, 8, true, kT, false>);
    else if (D % 32 == 0 && Dv % 32 == 0) launch(masked_decode_mfma_kernel<16, 8, true, kT, false>);
    else if (D <= 128) launch(masked_decode_mfma_kernel<8, 8, false, kT, false>);
    else launch(masked_decode_mfma_kernel<16, 8, false, kT, false>);
  };
  if (tied) sized(std::true_type{});
  else sized(std::false_type{});
  SEQ_CHECK_LAUNCH();
  if (n_split > 1) {
    hipLaunchKernelGGL(decode_split_join_kernel, dim3(T, H), dim3(WAVE), 0, SEQ_STREAM(),
                       (bf16raw*)out.data_ptr(), out.stride(0),
                       (const float*)part_o.data_ptr(), (const float*)part_ml.data_ptr(),
                       n_split, args);
    SEQ_CHECK_LAUNCH();
  }
  return true;
}
