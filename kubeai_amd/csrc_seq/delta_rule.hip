// Gated delta rule over the runs of a packed step. Per head a matrix state
// S [D, Dv] (fp32, one slot per sequence):
//
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// with q, k unit vectors per head (q times D^-1/2), beta = sigmoid(b),
// g = exp(-exp(a_log) softplus(a + dt_bias)): one number per head, or one per
// head and key channel, which then scales that channel's row of S (kChannel).
// Everything but the loads of q, k, v, a, b (serving dtype) is fp32. The value
// columns of a head are independent of each other, so a head is split over
// waves by column.
//
// Long runs are cut into segments that run in parallel. Over a segment the
// state goes S -> P S + B with P [D, D] the product of the tokens'
// (I - beta k k^T) diag(g) and B [D, Dv] what the segment writes from zero. Both
// come out of the same recurrence: B by walking from zero, P by walking the
// identity with zero values. Pass 1 (compose) walks every segment but the
// last for P and B, pass 2 (fold) chains S_(i+1) = P_i S_i + B_i per column
// block with P_i staged in LDS, pass 3 walks every segment from its incoming
// state and writes o.
#include "seq_common.h"
#include "delta_fold.h"

namespace {

constexpr int kTile = 16;  // tokens staged per barrier

DEV_INLINE float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// Any size: grid (n_seq * H, column blocks), block = the block's columns
// rounded up to a wave, that part of the head's state in LDS, thread j owns
// value column c0 + j.
template <typename T, bool kChannel>
__global__ void gated_delta_scan_kernel(
    float* __restrict__ o, const T* __restrict__ q, int64_t q_stride,
    const T* __restrict__ k, int64_t k_stride, const T* __restrict__ v,
    int64_t v_stride, const T* __restrict__ beta_pre, int64_t b_stride,
    const T* __restrict__ decay_pre, int64_t a_stride,
    const float* __restrict__ a_log, const float* __restrict__ dt_bias,
    float* __restrict__ state, const int* __restrict__ start_loc,
    const int* __restrict__ slots, const int* __restrict__ positions, int H, int G,
    int D, int Dv, int CB, float norm_eps) {
  const int s = blockIdx.x / H, h = blockIdx.x % H;
  const int hk = h / (H / G);
  const int s0 = start_loc[s], s1 = start_loc[s + 1], slot = slots[s];
  if (s1 <= s0) return;
  const int c0 = blockIdx.y * CB, nc = min(CB, Dv - c0);  // this block's columns
  extern __shared__ float sm[];
  float* S = sm;                      // [D][CB]
  float* qs = S + (size_t)D * CB;     // [tile][D]
  float* ks = qs + kTile * D;         // [tile][D]
  float* vs = ks + kTile * D;         // [tile][CB]
  float* gb = vs + kTile * CB;        // [tile][2]: decay, beta
  float* gs = gb + 2 * kTile;         // [tile][D]: decay per channel (kChannel)
  const int tid = threadIdx.x, nthr = blockDim.x;
  const bool carry = slot >= 0 && positions[s0] > 0;
  float* sp = state + ((size_t)(slot < 0 ? 0 : slot) * H + h) * D * Dv;
  for (int i = tid; i < D * CB; i += nthr) {
    const int r = i / CB, c = i % CB;
    S[i] = (carry && c < nc) ? sp[(size_t)r * Dv + c0 + c] : 0.f;
  }
  const float rate = -expf(a_log[h]), bias = kChannel ? 0.f : dt_bias[h];
  const float qscale = 1.0f / sqrtf((float)D);
  for (int t0 = s0; t0 < s1; t0 += kTile) {
    const int nt = min(kTile, s1 - t0);
    __syncthreads();  // the previous tile's readers are done
    for (int i = tid; i < nt * D; i += nthr) {
      const int tt = i / D, d = i % D;
      qs[i] = ldf(q + (size_t)(t0 + tt) * q_stride + hk * D + d);
      ks[i] = ldf(k + (size_t)(t0 + tt) * k_stride + hk * D + d);
      if constexpr (kChannel)
        gs[i] = expf(rate * softplus_f(ldf(decay_pre + (size_t)(t0 + tt) * a_stride + h * D + d) +
                                       dt_bias[h * D + d]));
    }
    for (int i = tid; i < nt * CB; i += nthr) {
      const int tt = i / CB, d = i % CB;
      vs[i] = d < nc ? ldf(v + (size_t)(t0 + tt) * v_stride + h * Dv + c0 + d) : 0.f;
    }
    __syncthreads();
    if (tid < nt) {
      float sq = 0.f, sk = 0.f;
      for (int d = 0; d < D; ++d) {
        sq += qs[tid * D + d] * qs[tid * D + d];
        sk += ks[tid * D + d] * ks[tid * D + d];
      }
      const float rq = qscale / sqrtf(sq + norm_eps), rk = 1.0f / sqrtf(sk + norm_eps);
      for (int d = 0; d < D; ++d) {
        qs[tid * D + d] *= rq;
        ks[tid * D + d] *= rk;
      }
      if constexpr (!kChannel) {
        const float a = ldf(decay_pre + (size_t)(t0 + tid) * a_stride + h);
        gb[2 * tid] = expf(rate * softplus_f(a + bias));
      }
      gb[2 * tid + 1] = sigmoid_f(ldf(beta_pre + (size_t)(t0 + tid) * b_stride + h));
    }
    __syncthreads();
    if (tid < nc) {
      for (int tt = 0; tt < nt; ++tt) {
        const float* qt = qs + tt * D;
        const float* kt = ks + tt * D;
        const float* gt = gs + tt * D;
        const float g = kChannel ? 1.f : gb[2 * tt], beta = gb[2 * tt + 1];
        float dot = 0.f;
        for (int i = 0; i < D; ++i) {
          const float st = (kChannel ? gt[i] : g) * S[i * CB + tid];
          S[i * CB + tid] = st;
          dot += st * kt[i];
        }
        const float u = beta * (vs[tt * CB + tid] - dot);
        float acc = 0.f;
        for (int i = 0; i < D; ++i) {
          const float st = S[i * CB + tid] + kt[i] * u;
          S[i * CB + tid] = st;
          acc += qt[i] * st;
        }
        o[((size_t)(t0 + tt) * H + h) * Dv + c0 + tid] = acc;
      }
    }
  }
  __syncthreads();
  if (slot >= 0)
    for (int i = tid; i < D * CB; i += nthr) {
      const int r = i / CB, c = i % CB;
      if (c < nc) sp[(size_t)r * Dv + c0 + c] = S[i];
    }
}

// exp(rate * softplus(x)) for rate <= 0, on the hardware's base-2 exponential
// and logarithm. ln(1 + e) = ln(u) * e / (u - 1) with u the rounded 1 + e keeps
// the relative accuracy of a softplus near zero, which is what a decay near one
// is made of.
DEV_INLINE float decay_f(float rate, float x) {
  constexpr float kL2e = 1.4426950408889634f, kLn2 = 0.6931471805599453f;
  const float e = __builtin_amdgcn_exp2f(x * kL2e);
  const float u = 1.f + e, d = u - 1.f;
  float sp = __builtin_amdgcn_logf(u) * kLn2 * (e * __builtin_amdgcn_rcpf(d));
  sp = d == 0.f ? e : sp;
  sp = x > 20.f ? x : sp;
  return __builtin_amdgcn_exp2f(rate * kL2e * sp);
}

// A wave is eight lane groups r = lane / 8 of eight lanes c; every lane brings
// partial sums x[0..3] of its group. Returns, in the 16-lane row e of the wave,
// the total of x[e] over the eight groups that share c.
DEV_INLINE float sum_to_rows(const float* x) {
  auto bits = [](float f) { return __builtin_bit_cast(unsigned, f); };
  auto flt = [](unsigned u) { return __builtin_bit_cast(float, u); };
  const auto a = __builtin_amdgcn_permlane32_swap(bits(x[0]), bits(x[2]), false, false);
  const auto b = __builtin_amdgcn_permlane32_swap(bits(x[1]), bits(x[3]), false, false);
  const float y0 = flt(a[0]) + flt(a[1]);  // halves of the wave: columns 0, 2
  const float y1 = flt(b[0]) + flt(b[1]);  // 1, 3
  const auto z = __builtin_amdgcn_permlane16_swap(bits(y0), bits(y1), false, false);
  const float t = flt(z[0]) + flt(z[1]);
  const int other = __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, t), 0x128, 0xf, 0xf,
                                                false);  // eight lanes on in the row
  return t + __builtin_bit_cast(float, other);
}

// the inverse way: row e's value in u[e] of every lane with the same c
DEV_INLINE void rows_to_all(float x, float* u) {
  const unsigned v = __builtin_bit_cast(unsigned, x);
  const auto a = __builtin_amdgcn_permlane16_swap(v, v, false, false);
  const auto even = __builtin_amdgcn_permlane32_swap(a[0], a[0], false, false);
  const auto odd = __builtin_amdgcn_permlane32_swap(a[1], a[1], false, false);
  u[0] = __builtin_bit_cast(float, (unsigned)even[0]);
  u[1] = __builtin_bit_cast(float, (unsigned)odd[0]);
  u[2] = __builtin_bit_cast(float, (unsigned)even[1]);
  u[3] = __builtin_bit_cast(float, (unsigned)odd[1]);
}

// the raw pieces of a row: four activations, or two where rows only divide so
template <typename T, int kN> struct RawN { typedef typename Raw4<T>::type type; };
template <> struct RawN<float, 2> { typedef float2 type; };
template <> struct RawN<bf16raw, 2> { typedef ushort2 type; };
DEV_INLINE void cvt_n(const float4& v, float* o) { cvt4(v, o); }
DEV_INLINE void cvt_n(const ushort4& v, float* o) { cvt4(v, o); }
DEV_INLINE void cvt_n(const float2& v, float* o) { o[0] = v.x; o[1] = v.y; }
DEV_INLINE void cvt_n(const ushort2& v, float* o) {
  o[0] = bf16_to_f32(v.x);
  o[1] = bf16_to_f32(v.y);
}

// kN floats to LDS, or from it, in the widest pieces that kN allows
template <int kN>
DEV_INLINE void lds_write_n(float* p, const float* x) {
  if constexpr (kN % 4 == 0) {
#pragma unroll
    for (int b = 0; b < kN; b += 4) st4(p + b, x + b);
  } else {
#pragma unroll
    for (int b = 0; b < kN; b += 2) *(float2*)(p + b) = make_float2(x[b], x[b + 1]);
  }
}

template <int kN>
DEV_INLINE void lds_read_n(const float* p, float* x) {
  if constexpr (kN % 4 == 0) {
#pragma unroll
    for (int b = 0; b < kN; b += 4) cvt4(*(const float4*)(p + b), x + b);
  } else {
#pragma unroll
    for (int b = 0; b < kN; b += 2) {
      const float2 v = *(const float2*)(p + b);
      x[b] = v.x;
      x[b + 1] = v.y;
    }
  }
}

constexpr int kCols = 4;  // value columns of a lane (register-state kernel)

// Register-state form for key sizes D = 16 * kQ (<= 128). One wave per block
// owns 32 columns of one head's state over one segment of one run: lane (r, c)
// of 8 x 8 keeps rows [r D/8, (r+1) D/8) of columns 4c..4c+3 in registers, so
// what a token brings (k, q, decays) is read from LDS once for four columns. A
// token costs two passes over the registers; the sums over a column's eight
// lanes (the dot with k before the write, the one with q after it) are lane
// swaps that leave one column's total to every lane. q, k of kTok tokens are staged through LDS, normalised once per
// token (and per-channel decays, activated once per token); the next tile is
// fetched into registers while the current one is walked.
//
// mode 0 (walk): columns are value columns; the segment starts from the
//   slot's state (first segment), or from seg_state[seg] (later ones);
//   writes o, and the slot's state after the run's last segment.
// mode 1 (compose): the first ceil(D / 32) column blocks are columns of
//   the identity walked with zero values (-> seg_p, stored transposed), the
//   rest value columns walked from zero (-> seg_b); the run's last segment is
//   skipped.
template <typename T, int kQ, bool kChannel>
__global__ __launch_bounds__(WAVE, 2) void gated_delta_scan_reg_kernel(
    float* __restrict__ o, const T* __restrict__ q, int64_t q_stride,
    const T* __restrict__ k, int64_t k_stride, const T* __restrict__ v,
    int64_t v_stride, const T* __restrict__ beta_pre, int64_t b_stride,
    const T* __restrict__ decay_pre, int64_t a_stride,
    const float* __restrict__ a_log, const float* __restrict__ dt_bias,
    float* __restrict__ state, const int* __restrict__ start_loc,
    const int* __restrict__ slots, const int* __restrict__ positions, int H, int G,
    int Dv, int ncb, float norm_eps, int nseg, int seg_len, int mode,
    float* __restrict__ seg_p, float* __restrict__ seg_b,
    const float* __restrict__ seg_state) {
  constexpr int D = 16 * kQ, R = D / 8, W = 8 * kCols;
  // tokens staged per barrier: with per-channel decays in LDS too, fewer, so that
  // LDS holds as many blocks as the registers do
  constexpr int kTok = kChannel ? 8 : 16;
  constexpr int kPart = WAVE / kTok, SR = D / kPart;  // lanes of a token, rows of a lane
  const int cb = blockIdx.x % ncb;
  const int h = (blockIdx.x / ncb) % H;
  const int seg = (blockIdx.x / (ncb * H)) % nseg;
  const int s = blockIdx.x / (ncb * H * nseg);
  const int hk = h / (H / G);
  const int r0 = start_loc[s], s1_run = start_loc[s + 1], slot = slots[s];
  const int s0 = r0 + seg * seg_len;
  const int s1 = min(s0 + seg_len, s1_run);
  if (s0 >= s1_run) return;
  const bool compose = mode == 1;
  if (compose && s1 == s1_run) return;
  __shared__ __attribute__((aligned(16))) float qs[kTok * D];
  __shared__ __attribute__((aligned(16))) float ks[kTok * D];
  __shared__ __attribute__((aligned(16))) float gs[kChannel ? kTok * D : 4];
  __shared__ __attribute__((aligned(16))) float db[kChannel ? D : 4];  // the head's dt_bias
  __shared__ __attribute__((aligned(16))) float vs[kTok * W];
  __shared__ float gb[kTok * 2];
  const int lane = threadIdx.x, r = lane >> 3, c = lane & 7;
  // compose: the first column blocks walk the identity
  const int pcb = compose ? (D + W - 1) / W : 0;
  const bool ident = cb < pcb;
  const int vc0 = (cb - pcb) * W;       // the block's first value column (when not ident)
  const int j0 = vc0 + kCols * c;       // the lane's
  const bool whole = Dv % kCols == 0;   // a lane's columns are aligned, all or none valid
  float S[kCols][R];
  auto load_cols = [&](const float* base) {
    const float* p = base + (size_t)r * R * Dv;
    if (whole && j0 < Dv) {
#pragma unroll
      for (int i = 0; i < R; ++i) {
        const float4 x = *(const float4*)(p + (size_t)i * Dv + j0);
        S[0][i] = x.x; S[1][i] = x.y; S[2][i] = x.z; S[3][i] = x.w;
      }
    } else {  // columns past the end repeat the last one and are never stored
#pragma unroll
      for (int i = 0; i < R; ++i)
#pragma unroll
        for (int e = 0; e < kCols; ++e) S[e][i] = p[(size_t)i * Dv + min(j0 + e, Dv - 1)];
    }
  };
  auto store_cols = [&](float* base) {
    float* p = base + (size_t)r * R * Dv + j0;
    if (j0 >= Dv) return;
    if (whole) {
#pragma unroll
      for (int i = 0; i < R; ++i)
        *(float4*)(p + (size_t)i * Dv) = make_float4(S[0][i], S[1][i], S[2][i], S[3][i]);
    } else {
#pragma unroll
      for (int e = 0; e < kCols; ++e)
        if (j0 + e < Dv) {
#pragma unroll
          for (int i = 0; i < R; ++i) p[(size_t)i * Dv + e] = S[e][i];
        }
    }
  };
  const size_t head_at = ((size_t)(slot < 0 ? 0 : slot) * H + h) * D * Dv;
  if (!compose && seg > 0) {
    load_cols(seg_state + (((size_t)s * nseg + seg) * H + h) * D * Dv);
  } else if (!compose && slot >= 0 && positions[r0] > 0) {
    load_cols(state + head_at);
  } else {
#pragma unroll
    for (int e = 0; e < kCols; ++e)
#pragma unroll
      for (int i = 0; i < R; ++i)
        S[e][i] = (ident && r * R + i == cb * W + kCols * c + e) ? 1.f : 0.f;
  }
  const float rate = -expf(a_log[h]), bias = kChannel ? 0.f : dt_bias[h];
  const float qscale = 1.0f / sqrtf((float)D);
  // staging: lane (st_tt, st_part) owns SR rows of one token of the tile, in
  // pieces of VN elements
  constexpr int VN = SR % 4 == 0 ? 4 : 2, NV = SR / VN;
  typedef typename RawN<T, VN>::type rawn;
  typedef typename Raw4<T>::type raw4;
  constexpr int kPieces = kTok * D / 4;  // of four decays, dealt over the wave
  constexpr int NG = (kPieces + WAVE - 1) / WAVE;
  const int st_tt = lane / kPart, st_part = lane % kPart;
  rawn pq[NV], pk[NV];
  raw4 pg[kChannel ? NG : 1];
  T pv[W / kPart], pa, pb;
  // (tokens past the end repeat the last one, columns past the end too: what
  // they stage is never used)
  auto prefetch = [&](int tile0) {
    const int t = min(tile0 + st_tt, s1 - 1);
    const T* qp = q + (size_t)t * q_stride + hk * D + st_part * SR;
    const T* kp = k + (size_t)t * k_stride + hk * D + st_part * SR;
#pragma unroll
    for (int n = 0; n < NV; ++n) {
      pq[n] = *(const rawn*)(qp + VN * n);
      pk[n] = *(const rawn*)(kp + VN * n);
    }
    const T* vp = v + (size_t)t * v_stride + h * Dv;
#pragma unroll
    for (int e = 0; e < W / kPart; ++e)
      pv[e] = vp[max(0, min(vc0 + st_part * (W / kPart) + e, Dv - 1))];
    if constexpr (!kChannel) pa = decay_pre[(size_t)t * a_stride + h];
    pb = beta_pre[(size_t)t * b_stride + h];
    if constexpr (kChannel) {
#pragma unroll
      for (int n = 0; n < NG; ++n) {
        const int w = n * WAVE + lane, tt = w / (D / 4), d = w % (D / 4) * 4;
        if (tile0 + n * WAVE / (D / 4) < s1)  // wave-uniform
          pg[n] = *(const raw4*)(decay_pre + (size_t)min(tile0 + tt, s1 - 1) * a_stride +
                                 h * D + d);
      }
    }
  };
  prefetch(s0);
  if constexpr (kChannel)
    for (int d = lane; d < D; d += WAVE) db[d] = dt_bias[(size_t)h * D + d];
  for (int t0 = s0; t0 < s1; t0 += kTok) {
    const int nt = min(kTok, s1 - t0);
    __syncthreads();
    {
      float qa[SR], ka[SR];
      float sq = 0.f, sk = 0.f;
#pragma unroll
      for (int n = 0; n < NV; ++n) {
        cvt_n(pq[n], qa + VN * n);
        cvt_n(pk[n], ka + VN * n);
      }
#pragma unroll
      for (int i = 0; i < SR; ++i) {
        sq += qa[i] * qa[i];
        sk += ka[i] * ka[i];
      }
      // the lanes of a token are neighbours
#pragma unroll
      for (int x = 1; x < kPart; x *= 2) {
        sq += __shfl_xor(sq, x, WAVE);
        sk += __shfl_xor(sk, x, WAVE);
      }
      const float rq = qscale / sqrtf(sq + norm_eps), rk = 1.0f / sqrtf(sk + norm_eps);
#pragma unroll
      for (int i = 0; i < SR; ++i) {
        qa[i] *= rq;
        ka[i] *= rk;
      }
      lds_write_n<SR>(qs + st_tt * D + st_part * SR, qa);
      lds_write_n<SR>(ks + st_tt * D + st_part * SR, ka);
#pragma unroll
      for (int e = 0; e < W / kPart; ++e)
        vs[st_tt * W + st_part * (W / kPart) + e] = ident ? 0.f : ldf(&pv[e]);
      if (st_part == 0) {
        if constexpr (!kChannel) gb[2 * st_tt] = expf(rate * softplus_f(ldf(&pa) + bias));
        gb[2 * st_tt + 1] = sigmoid_f(ldf(&pb));
      }
      if constexpr (kChannel) {
#pragma unroll
        for (int n = 0; n < NG; ++n) {
          const int w = n * WAVE + lane, d = w % (D / 4) * 4;
          if (n * WAVE / (D / 4) < nt && (kPieces % WAVE == 0 || w < kPieces)) {
            float x[4];
            cvt4(pg[n], x);
            const float4 bd = *(const float4*)(db + d);
            *(float4*)(gs + 4 * w) =
                make_float4(decay_f(rate, x[0] + bd.x), decay_f(rate, x[1] + bd.y),
                            decay_f(rate, x[2] + bd.z), decay_f(rate, x[3] + bd.w));
          }
        }
      }
    }
    __syncthreads();
    if (t0 + kTok < s1) prefetch(t0 + kTok);
    for (int tt = 0; tt < nt; ++tt) {
      const float vj = vs[tt * W + kCols * c + (lane >> 4)];  // the lane's total's column
      const float beta = gb[2 * tt + 1];
      float ka[R], ga[kChannel ? R : 1], qa[R];
      lds_read_n<R>(ks + tt * D + r * R, ka);
      if constexpr (kChannel) lds_read_n<R>(gs + tt * D + r * R, ga);
      lds_read_n<R>(qs + tt * D + r * R, qa);
      const float g = kChannel ? 1.f : gb[2 * tt];
      float dot[kCols] = {0.f, 0.f, 0.f, 0.f}, u[kCols];
#pragma unroll
      for (int i = 0; i < R; ++i)
#pragma unroll
        for (int e = 0; e < kCols; ++e) {
          S[e][i] *= kChannel ? ga[kChannel ? i : 0] : g;
          dot[e] += S[e][i] * ka[i];
        }
      rows_to_all(beta * (vj - sum_to_rows(dot)), u);
      float acc[kCols] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < R; ++i)
#pragma unroll
        for (int e = 0; e < kCols; ++e) {
          S[e][i] += ka[i] * u[e];
          acc[e] += qa[i] * S[e][i];
        }
      if (!compose) {
        const float total = sum_to_rows(acc);
        const int col = j0 + (lane >> 4);
        if ((lane & 8) == 0 && col < Dv) o[((size_t)(t0 + tt) * H + h) * Dv + col] = total;
      }
    }
  }
  if (compose) {
    const size_t sh = ((size_t)s * nseg + seg) * H + h;
    if (ident) {
#pragma unroll
      for (int e = 0; e < kCols; ++e) {
        const int col = cb * W + kCols * c + e;
        float* pp = seg_p + sh * D * D + (size_t)col * D + r * R;  // P^T
        if (col < D) {
#pragma unroll
          for (int i = 0; i < R; i += 2) *(float2*)(pp + i) = make_float2(S[e][i], S[e][i + 1]);
        }
      }
    } else {
      store_cols(seg_b + sh * D * Dv);
    }
  } else if (slot >= 0 && s1 == s1_run) {
    store_cols(state + head_at);
  }
}

}  // namespace

#define DELTA_CASE(KQ)                                              \
  case KQ:                                                          \
    if (channel) launch(gated_delta_scan_reg_kernel<act_t, KQ, true>);  \
    else launch(gated_delta_scan_reg_kernel<act_t, KQ, false>);     \
    break;

void gated_delta_scan(torch::Tensor o, torch::Tensor q, torch::Tensor k,
                      torch::Tensor v, torch::Tensor beta_pre, torch::Tensor decay_pre,
                      torch::Tensor a_log, torch::Tensor dt_bias, torch::Tensor state,
                      torch::Tensor start_loc, torch::Tensor slots,
                      torch::Tensor positions, double norm_eps, int64_t max_len) {
  check_f32(o, "o");
  check_f32(state, "state");
  check_f32(a_log, "a_log");
  check_f32(dt_bias, "dt_bias");
  check_i32(start_loc, "start_loc");
  check_i32(slots, "slots");
  check_i32(positions, "positions");
  check_rows(beta_pre, "beta_pre");
  // decay per head [T, H], or per head and key channel [T, H, D]
  const bool channel = decay_pre.dim() == 3;
  if (!channel) check_rows(decay_pre, "decay_pre");
  TORCH_CHECK(q.dim() == 3 && k.dim() == 3 && v.dim() == 3 && q.is_cuda());
  const int T = q.size(0), G = q.size(1), D = q.size(2), H = v.size(1), Dv = v.size(2);
  auto dense_heads = [](const torch::Tensor& t) {
    return t.stride(2) == 1 && (t.size(1) == 1 || t.stride(1) == t.size(2));
  };
  TORCH_CHECK(dense_heads(q) && dense_heads(k) && dense_heads(v),
              "q/k/v heads must be dense within a row");
  TORCH_CHECK(k.size(0) == T && k.size(1) == G && k.size(2) == D && v.size(0) == T);
  TORCH_CHECK(G > 0 && H % G == 0, "value heads must be a multiple of q/k heads");
  TORCH_CHECK(k.scalar_type() == q.scalar_type() && v.scalar_type() == q.scalar_type() &&
              beta_pre.scalar_type() == q.scalar_type() &&
              decay_pre.scalar_type() == q.scalar_type());
  TORCH_CHECK(beta_pre.size(0) == T && beta_pre.size(1) == H && decay_pre.size(0) == T &&
              decay_pre.size(1) == H && a_log.numel() == H && decay_pre.is_cuda());
  TORCH_CHECK(dt_bias.numel() == (channel ? (int64_t)H * D : H));
  TORCH_CHECK(!channel || (decay_pre.size(2) == D && dense_heads(decay_pre)),
              "decays per channel must be laid out heads x key size");
  TORCH_CHECK(o.size(0) == T && o.size(1) == H && o.size(2) == Dv);
  TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == D &&
              state.size(3) == Dv);
  TORCH_CHECK(start_loc.numel() == slots.numel() + 1 && positions.numel() == T);
  const int n_seq = slots.numel();
  if (n_seq == 0 || T == 0) return;
  auto vec_ok = [&](const torch::Tensor& t) {
    const size_t bytes = 4 * t.element_size();
    return ((size_t)t.data_ptr()) % bytes == 0 && t.stride(0) % 4 == 0;
  };
  if (D % 16 == 0 && D <= 128 && vec_ok(q) && vec_ok(k) && (!channel || vec_ok(decay_pre))) {
    constexpr int W = 8 * kCols;
    const int ncb = (Dv + W - 1) / W;
    int seg_len, nseg;
    delta_segments(max_len, n_seq, H, D, Dv, &seg_len, &nseg);
    torch::Tensor ws_p, ws_b, ws_s;
    if (nseg > 1) {
      ws_p = torch::empty({(int64_t)n_seq * nseg * H * D * D}, state.options());
      ws_b = torch::empty({(int64_t)n_seq * nseg * H * D * Dv}, state.options());
      ws_s = torch::empty({(int64_t)n_seq * nseg * H * D * Dv}, state.options());
    }
    SEQ_DISPATCH_ACT(q, {
      auto launch1 = [&](auto kern, int mode) {
        const int blocks_cb = mode == 1 ? ncb + (D + W - 1) / W : ncb;
        hipLaunchKernelGGL(kern, dim3(n_seq * nseg * H * blocks_cb), dim3(WAVE), 0,
                           SEQ_STREAM(), (float*)o.data_ptr(),
                           (const act_t*)q.data_ptr(), q.stride(0),
                           (const act_t*)k.data_ptr(), k.stride(0),
                           (const act_t*)v.data_ptr(), v.stride(0),
                           (const act_t*)beta_pre.data_ptr(), beta_pre.stride(0),
                           (const act_t*)decay_pre.data_ptr(), decay_pre.stride(0),
                           (const float*)a_log.data_ptr(),
                           (const float*)dt_bias.data_ptr(), (float*)state.data_ptr(),
                           (const int*)start_loc.data_ptr(),
                           (const int*)slots.data_ptr(),
                           (const int*)positions.data_ptr(), H, G, Dv, blocks_cb,
                           (float)norm_eps, nseg, seg_len, mode,
                           nseg > 1 ? (float*)ws_p.data_ptr() : nullptr,
                           nseg > 1 ? (float*)ws_b.data_ptr() : nullptr,
                           nseg > 1 ? (const float*)ws_s.data_ptr() : nullptr);
      };
      auto launch = [&](auto kern) {
        if (nseg > 1) {
          launch1(kern, 1);
          delta_fold_launch(D, n_seq, H, Dv, nseg, seg_len, ws_s, ws_p, ws_b, state,
                            start_loc, slots, positions);
        }
        launch1(kern, 0);
      };
      switch (D / 16) {
        DELTA_CASE(1) DELTA_CASE(2) DELTA_CASE(3) DELTA_CASE(4)
        DELTA_CASE(5) DELTA_CASE(6) DELTA_CASE(7) DELTA_CASE(8)
      }
    });
    SEQ_CHECK_LAUNCH();
    return;
  }
  // value columns per block: all of them if the state fits LDS, else fewer
  // (columns are independent), in whole waves
  auto lds_for = [&](int cb) {
    return ((size_t)D * cb + (channel ? 3 : 2) * kTile * D + (size_t)kTile * cb + 2 * kTile) *
           sizeof(float);
  };
  int CB = std::min(((Dv + WAVE - 1) / WAVE) * WAVE, 1024);
  while (CB > WAVE && lds_for(CB) > 144 * 1024) CB -= WAVE;
  const size_t lds = lds_for(CB);
  TORCH_CHECK(lds <= 160 * 1024, "key size too large for the LDS state");
  const int threads = CB, ncb_gen = (Dv + CB - 1) / CB;
  TORCH_CHECK(ncb_gen <= 65535);
  SEQ_DISPATCH_ACT(q, {
    auto kern = channel ? gated_delta_scan_kernel<act_t, true>
                        : gated_delta_scan_kernel<act_t, false>;
    // raise the dynamic-LDS cap once per kernel, outside any capture
    static thread_local const void* raised[4] = {nullptr, nullptr, nullptr, nullptr};
    if (lds > 48 * 1024) {
      bool seen = false;
      for (auto p : raised) seen |= p == (const void*)kern;
      if (!seen) {
        hipFuncSetAttribute((const void*)kern,
                            hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
        for (auto& p : raised)
          if (p == nullptr) { p = (const void*)kern; break; }
      }
    }
    hipLaunchKernelGGL(kern, dim3(n_seq * H, ncb_gen), dim3(threads), lds, SEQ_STREAM(),
                       (float*)o.data_ptr(), (const act_t*)q.data_ptr(), q.stride(0),
                       (const act_t*)k.data_ptr(), k.stride(0),
                       (const act_t*)v.data_ptr(), v.stride(0),
                       (const act_t*)beta_pre.data_ptr(), beta_pre.stride(0),
                       (const act_t*)decay_pre.data_ptr(), decay_pre.stride(0),
                       (const float*)a_log.data_ptr(), (const float*)dt_bias.data_ptr(),
                       (float*)state.data_ptr(), (const int*)start_loc.data_ptr(),
                       (const int*)slots.data_ptr(), (const int*)positions.data_ptr(), H,
                       G, D, Dv, CB, (float)norm_eps);
  });
  SEQ_CHECK_LAUNCH();
}
