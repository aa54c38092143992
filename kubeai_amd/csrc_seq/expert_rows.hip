// Routing of tokens to experts in one step, and the bookkeeping of gathered
// expert rows: a stable sort of (token, choice) pairs by expert and the sum of
// a token's rows afterwards.
#include "seq_common.h"

namespace {

constexpr int kRW = 4;   // waves of a routing block
constexpr int kEB = 8;   // experts accumulated at a time

// A wave routes TPW tokens: logits of all rows of the router (fp32 products,
// N channels a lane and step), scores = softmax or sigmoid of the first E, the
// `top` largest s + bias in the order (value descending, index ascending),
// weights s * wscale. LDS holds the wave's logits, then scores [TPW][R].
// kJoint (few tokens): the block's waves share one token's channels, and the
// first wave routes it.
template <typename T, int TPW, bool kVec, bool kJoint>
__global__ __launch_bounds__(kRW * WAVE) void route_tokens_kernel(
    const T* __restrict__ h, int64_t h_stride, const float* __restrict__ router,
    const float* __restrict__ bias, float* __restrict__ dense,
    float* __restrict__ weights, int* __restrict__ index, float* __restrict__ extra,
    int n_tok, int C, int E, int R, int top, float wscale, int sigmoid) {
  constexpr int N = kVec ? Vec16<T>::N : 1;
  extern __shared__ float lds[];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  const int t0 = kJoint ? blockIdx.x : (blockIdx.x * kRW + wave) * TPW;
  if (t0 >= n_tok) return;  // a whole wave (kJoint: never)
  float* z = lds + (size_t)wave * TPW * R;
  const int c_first = (kJoint ? wave * WAVE + lane : lane) * N;
  const int c_step = (kJoint ? kRW : 1) * WAVE * N;
  const int nt = min(TPW, n_tok - t0);
  for (int e0 = 0; e0 < R; e0 += kEB) {
    float acc[TPW][kEB];
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int e = 0; e < kEB; ++e) acc[i][e] = 0.f;
    for (int c = c_first; c < C; c += c_step) {
      float x[TPW][N];
#pragma unroll
      for (int i = 0; i < TPW; ++i) {
        const T* hp = h + (size_t)(t0 + min(i, nt - 1)) * h_stride + c;
        if constexpr (kVec) Vec16<T>::load(hp, x[i]);
        else x[i][0] = ldf(hp);
      }
#pragma unroll
      for (int e = 0; e < kEB; ++e) {
        const float* wp = router + (size_t)min(e0 + e, R - 1) * C + c;
        float w[N];
        if constexpr (kVec) {
#pragma unroll
          for (int j = 0; j < N; j += 4) {
            const float4 v = *(const float4*)(wp + j);
            w[j] = v.x; w[j + 1] = v.y; w[j + 2] = v.z; w[j + 3] = v.w;
          }
        } else {
          w[0] = *wp;
        }
#pragma unroll
        for (int i = 0; i < TPW; ++i)
#pragma unroll
          for (int j = 0; j < N; ++j) acc[i][e] = fmaf(x[i][j], w[j], acc[i][e]);
      }
    }
#pragma unroll
    for (int i = 0; i < TPW; ++i)
#pragma unroll
      for (int e = 0; e < kEB; ++e) {
        const float s = wave_sum(acc[i][e]);
        if (lane == 0 && e0 + e < R) z[i * R + e0 + e] = s;
      }
  }
  if constexpr (kJoint) {
    __syncthreads();
    if (wave > 0) return;
    for (int e = lane; e < R; e += WAVE) {
      float s = z[e];
      for (int w = 1; w < kRW; ++w) s += lds[(size_t)w * R + e];
      z[e] = s;
    }
  }
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
  for (int i = 0; i < nt; ++i) {
    const int t = t0 + i;
    float* s = z + i * R;
    if (extra != nullptr)
      for (int e = E + lane; e < R; e += WAVE) extra[(size_t)t * (R - E) + e - E] = s[e];
    if (sigmoid) {
      for (int e = lane; e < E; e += WAVE) s[e] = sigmoid_f(s[e]);
    } else {
      float zmax = -INFINITY, sum = 0.f;
      for (int e = lane; e < E; e += WAVE) zmax = fmaxf(zmax, s[e]);
      zmax = wave_max(zmax);
      for (int e = lane; e < E; e += WAVE) {
        const float p = expf(s[e] - zmax);
        s[e] = p;
        sum += p;
      }
      sum = wave_sum(sum);
      for (int e = lane; e < E; e += WAVE) s[e] = s[e] / sum;
    }
    for (int e = lane; e < E; e += WAVE) dense[(size_t)t * E + e] = 0.f;
    float last_v = INFINITY;
    int last_i = -1;
    for (int k = 0; k < top; ++k) {
      float bv = -INFINITY;
      int bi = E;  // none
      for (int e = lane; e < E; e += WAVE) {
        const float v = s[e] + (bias != nullptr ? bias[e] : 0.f);
        const bool after = v < last_v || (v == last_v && e > last_i);
        if (after && (bi == E || v > bv)) {
          bv = v;
          bi = e;
        }
      }
#pragma unroll
      for (int off = 32; off > 0; off >>= 1) {
        const float ov = __shfl_xor(bv, off, WAVE);
        const int oi = __shfl_xor(bi, off, WAVE);
        const bool take = oi < E && (bi == E || ov > bv || (ov == bv && oi < bi));
        bv = take ? ov : bv;
        bi = take ? oi : bi;
      }
      if (bi == E) bi = 0;  // NaN scores: stay in range
      last_v = bv;
      last_i = bi;
      if (lane == 0) {
        const float w = s[bi] * wscale;
        weights[(size_t)t * top + k] = w;
        index[(size_t)t * top + k] = bi;
      }
      // the lane that cleared the column sets it
      if (lane == bi % WAVE) dense[(size_t)t * E + bi] = s[bi] * wscale;
    }
  }
}

constexpr int kSB = 1024;  // threads of a sorting block

// grid (E): block e places the pairs of expert e. Its first place is the
// number of pairs of lower experts; a pair's rank is the number of earlier
// pairs of the same expert (block-wide prefix sums over slices of the list).
__global__ __launch_bounds__(kSB) void expert_order_kernel(
    const int* __restrict__ index, const float* __restrict__ weights,
    int* __restrict__ tok, float* __restrict__ wrow, int* __restrict__ place,
    int* __restrict__ counts, int N, int top) {
  __shared__ int part[kSB / WAVE + 1], total_s;
  const int e = blockIdx.x;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x % WAVE;
  int below = 0;
  for (int i = threadIdx.x; i < N; i += kSB) below += index[i] < e ? 1 : 0;
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) below += __shfl_xor(below, off, WAVE);
  if (lane == 0) part[wave] = below;
  __syncthreads();
  if (threadIdx.x == 0) {
    int s = 0;
    for (int w = 0; w < kSB / WAVE; ++w) s += part[w];
    total_s = s;
  }
  __syncthreads();
  const int first = total_s;
  int at = first;
  for (int i0 = 0; i0 < N; i0 += kSB) {
    const int i = i0 + threadIdx.x;
    const bool mine = i < N && index[i] == e;
    const uint64_t b = __ballot(mine);
    __syncthreads();  // the previous slice's counts have been read
    if (lane == 0) part[wave] = __popcll(b);
    __syncthreads();
    int before = 0, all = 0;
    for (int w = 0; w < kSB / WAVE; ++w) {
      if (w < wave) before += part[w];
      all += part[w];
    }
    if (mine) {
      const int p = at + before + __popcll(b & ((1ull << lane) - 1));
      tok[p] = i / top;
      wrow[p] = weights[i];
      place[i] = p;
    }
    at += all;
  }
  if (threadIdx.x == 0) counts[e] = at - first;
}

// grid (T, channel blocks): out[t] = sum_k y[place[t, k]] (+ shared[t]), fp32
template <typename T, bool kVec>
__global__ __launch_bounds__(256) void combine_rows_kernel(
    T* __restrict__ out, const T* __restrict__ y, const int* __restrict__ place,
    const T* __restrict__ shared, int C, int top) {
  constexpr int N = kVec ? Vec16<T>::N : 1;
  const int t = blockIdx.x;
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * N;
  if (c >= C) return;
  auto load = [](const T* p, float* x) {
    if constexpr (kVec) Vec16<T>::load(p, x);
    else x[0] = ldf(p);
  };
  float acc[N], x[N];
#pragma unroll
  for (int e = 0; e < N; ++e) acc[e] = 0.f;
  for (int k = 0; k < top; ++k) {
    load(y + (size_t)place[(size_t)t * top + k] * C + c, x);
#pragma unroll
    for (int e = 0; e < N; ++e) acc[e] += x[e];
  }
  if (shared != nullptr) {
    load(shared + (size_t)t * C + c, x);
#pragma unroll
    for (int e = 0; e < N; ++e) acc[e] += x[e];
  }
  if constexpr (kVec) Vec16<T>::store(out + (size_t)t * C + c, acc);
  else stf(out + (size_t)t * C + c, acc[0]);
}

}  // namespace

void route_tokens(torch::Tensor h, torch::Tensor router, c10::optional<torch::Tensor> bias,
                  torch::Tensor dense, torch::Tensor weights, torch::Tensor index,
                  c10::optional<torch::Tensor> extra, double scale, int64_t score) {
  check_rows(h, "h");
  check_f32(router, "router");
  check_f32(dense, "dense");
  check_f32(weights, "weights");
  check_i32(index, "index");
  TORCH_CHECK(score == 0 || score == 1, "score: 0 softmax, 1 sigmoid");
  TORCH_CHECK(router.dim() == 2 && dense.dim() == 2 && weights.dim() == 2);
  const int T = h.size(0), C = h.size(1), R = router.size(0), E = dense.size(1);
  const int top = weights.size(1);
  TORCH_CHECK(router.size(1) == C && E >= 1 && E <= R && dense.size(0) == T);
  TORCH_CHECK(top >= 1 && top <= E && weights.size(0) == T && index.numel() == (int64_t)T * top,
              "top must be within the number of experts");
  TORCH_CHECK(extra.has_value() == (R > E));
  if (extra.has_value()) {
    check_f32(*extra, "extra");
    TORCH_CHECK(extra->numel() == (int64_t)T * (R - E));
  }
  if (bias.has_value()) {
    check_f32(*bias, "bias");
    TORCH_CHECK(bias->numel() == E);
  }
  if (T == 0) return;
  // several tokens a wave share the router's rows; few tokens take a block each
  const bool joint = T <= 1024;
  const int tpw = joint ? 1 : 4;
  const size_t lds = (size_t)kRW * tpw * R * 4;
  TORCH_CHECK(lds <= 64 * 1024, "too many experts");
  const int per = joint ? 1 : kRW * tpw;
  SEQ_DISPATCH_ACT(h, {
    constexpr int n = Vec16<act_t>::N;
    const bool vec = C % n == 0 && h.stride(0) % n == 0 && ((size_t)h.data_ptr()) % 16 == 0 &&
                     ((size_t)router.data_ptr()) % 16 == 0;
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3((T + per - 1) / per), dim3(kRW * WAVE), lds, SEQ_STREAM(),
                         (const act_t*)h.data_ptr(), h.stride(0),
                         (const float*)router.data_ptr(),
                         bias.has_value() ? (const float*)bias->data_ptr() : nullptr,
                         (float*)dense.data_ptr(), (float*)weights.data_ptr(),
                         (int*)index.data_ptr(),
                         extra.has_value() ? (float*)extra->data_ptr() : nullptr, T, C, E, R,
                         top, (float)scale, (int)score);
    };
    if (vec && joint) launch(route_tokens_kernel<act_t, 1, true, true>);
    else if (vec) launch(route_tokens_kernel<act_t, 4, true, false>);
    else if (joint) launch(route_tokens_kernel<act_t, 1, false, true>);
    else launch(route_tokens_kernel<act_t, 4, false, false>);
  });
  SEQ_CHECK_LAUNCH();
}

void expert_order(torch::Tensor index, torch::Tensor weights, torch::Tensor tok,
                  torch::Tensor wrow, torch::Tensor place, torch::Tensor counts) {
  check_i32(index, "index");
  check_f32(weights, "weights");
  check_i32(tok, "tok");
  check_f32(wrow, "wrow");
  check_i32(place, "place");
  check_i32(counts, "counts");
  TORCH_CHECK(index.dim() == 2);
  const int64_t N = index.numel();
  TORCH_CHECK(weights.numel() == N && tok.numel() == N && wrow.numel() == N &&
              place.numel() == N && N < (int64_t)1 << 30 && counts.numel() >= 1);
  if (N == 0) return;
  hipLaunchKernelGGL(expert_order_kernel, dim3(counts.numel()), dim3(kSB), 0, SEQ_STREAM(),
                     (const int*)index.data_ptr(), (const float*)weights.data_ptr(),
                     (int*)tok.data_ptr(), (float*)wrow.data_ptr(), (int*)place.data_ptr(),
                     (int*)counts.data_ptr(), (int)N, (int)index.size(1));
  SEQ_CHECK_LAUNCH();
}

void combine_expert_rows(torch::Tensor out, torch::Tensor y, torch::Tensor place,
                         c10::optional<torch::Tensor> shared) {
  check_i32(place, "place");
  TORCH_CHECK(out.is_cuda() && y.is_cuda() && out.is_contiguous() && y.is_contiguous() &&
              out.dim() == 2 && y.dim() == 2 && place.dim() == 2);
  const int T = out.size(0), C = out.size(1), top = place.size(1);
  TORCH_CHECK(y.size(1) == C && place.size(0) == T && y.size(0) == place.numel() &&
              y.scalar_type() == out.scalar_type());
  const void* sp = nullptr;
  if (shared.has_value()) {
    TORCH_CHECK(shared->is_cuda() && shared->is_contiguous() && shared->sizes() == out.sizes() &&
                shared->scalar_type() == out.scalar_type());
    sp = shared->data_ptr();
  }
  if (T == 0 || C == 0) return;
  const int n = 16 / y.element_size();
  const bool vec = C % n == 0 && ((size_t)y.data_ptr()) % 16 == 0 &&
                   ((size_t)out.data_ptr()) % 16 == 0 && ((size_t)sp) % 16 == 0;
  const int per = 256 * (vec ? n : 1);
  TORCH_CHECK((C + per - 1) / per <= 65535);
  SEQ_DISPATCH_ACT(y, {
    auto launch = [&](auto kern) {
      hipLaunchKernelGGL(kern, dim3(T, (C + per - 1) / per), dim3(256), 0, SEQ_STREAM(),
                         (act_t*)out.data_ptr(), (const act_t*)y.data_ptr(),
                         (const int*)place.data_ptr(), (const act_t*)sp, C, top);
    };
    if (vec) launch(combine_rows_kernel<act_t, true>);
    else launch(combine_rows_kernel<act_t, false>);
  });
  SEQ_CHECK_LAUNCH();
}
