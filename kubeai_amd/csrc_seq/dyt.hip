// Dynamic tanh, dyt(x) = tanh(alpha x) * w + b, around a sublayer, fused with
// the residual add and the causal input convolution of the next sublayer. The
// norm has no statistics, so a channel never needs its neighbours: a thread
// walks tokens of a few channels with the convolution's window in registers.
#include "seq_common.h"

namespace {

constexpr int kMaxConvTail = 15;  // taps - 1

struct DytParams {
  const float *alpha, *w, *b;
};

template <int V> DEV_INLINE void load_f(const float* p, float* x) {
  if constexpr (V == 4) {
    const float4 v = *(const float4*)p;
    x[0] = v.x; x[1] = v.y; x[2] = v.z; x[3] = v.w;
  } else {
    x[0] = *p;
  }
}
template <int V, typename T> DEV_INLINE void load_act(const T* p, float* x) {
  if constexpr (V == 4) cvt4(*(const typename Raw4<T>::type*)p, x);
  else x[0] = ldf(p);
}
template <int V> DEV_INLINE void store_act(float* p, const float* x) {
  if constexpr (V == 4) *(float4*)p = make_float4(x[0], x[1], x[2], x[3]);
  else *p = x[0];
}
template <int V> DEV_INLINE void store_act(bf16raw* p, const float* x) {
  if constexpr (V == 4) {
    ushort4 v;
    v.x = f32_to_bf16(x[0]); v.y = f32_to_bf16(x[1]);
    v.z = f32_to_bf16(x[2]); v.w = f32_to_bf16(x[3]);
    *(ushort4*)p = v;
  } else {
    *p = f32_to_bf16(x[0]);
  }
}

// grid (token spans, channel blocks); a thread owns V channels of `span`
// consecutive tokens of the packed stream:
//   r' = r + dyt_post(branch),  h = dyt_pre(r'),  out = h + sum_j conv[j] h_(t-K1+j)
// TAIL bounds taps - 1; the window is kept zero-padded to TAIL entries. Inputs
// ahead of a span come from their run's own tokens (formed again: r is read,
// not updated in place), inputs ahead of a run from its carried tail;
// positions < 0 are 0. A run inside one span advances its tail here; the
// others leave that to dyt_tail_kernel, since their first span may still be
// reading it.
template <typename T, typename B, int V, int TAIL>
__global__ __launch_bounds__(128) void add_dyt_conv_kernel(
    T* __restrict__ out, float* __restrict__ r_out, const B* __restrict__ branch,
    DytParams post, const float* __restrict__ r_in, DytParams pre,
    const float* __restrict__ conv_w, float* __restrict__ tails,
    const int* __restrict__ start_loc, const int* __restrict__ slots,
    const int* __restrict__ token_seq, const int* __restrict__ positions, int T_all,
    int C, int K1, int span) {
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * V;
  const int t0 = blockIdx.x * span, t1 = min(T_all, t0 + span);
  if (c >= C) return;
  const float al = pre.alpha[0], alp = branch != nullptr ? post.alpha[0] : 0.f;
  float w[V], b[V], pw[V], pb[V];
  load_f<V>(pre.w + c, w);
  load_f<V>(pre.b + c, b);
  if (branch != nullptr) {
    load_f<V>(post.w + c, pw);
    load_f<V>(post.b + c, pb);
  }
  auto residual = [&](int t, float* x) {
    load_f<V>(r_in + (size_t)t * C + c, x);
    if (branch != nullptr) {
      float y[V];
      load_act<V>(branch + (size_t)t * C + c, y);
#pragma unroll
      for (int e = 0; e < V; ++e) x[e] += fmaf(tanh_f(alp * y[e]), pw[e], pb[e]);
    }
  };
  auto squash = [&](const float* x, float* h) {
#pragma unroll
    for (int e = 0; e < V; ++e) h[e] = fmaf(tanh_f(al * x[e]), w[e], b[e]);
  };
  // cw[TAIL] meets the current token, cw[TAIL - d] the token d steps back
  float cw[TAIL + 1][V], hist[TAIL > 0 ? TAIL : 1][V];
#pragma unroll
  for (int j = 0; j <= TAIL; ++j)
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const int tap = j - (TAIL - K1);
      cw[j][e] = conv_w != nullptr && tap >= 0
                     ? conv_w[(size_t)(c + e) * (K1 + 1) + tap] : 0.f;
    }
  int s0 = 0, s1 = 0, slot = -1;  // the run that token t lies in
  auto enter_run = [&](int t) {
    const int s = token_seq[t];
    s0 = start_loc[s];
    s1 = start_loc[s + 1];
    slot = slots[s];
    const int p0 = positions[s0];
#pragma unroll
    for (int i = 0; i < TAIL; ++i) {
      const int d = TAIL - i;  // steps back from t
      const int tb = t - d;
#pragma unroll
      for (int e = 0; e < V; ++e) hist[i][e] = 0.f;
      if (d > K1) continue;
      if (tb >= s0) {
        float x[V];
        residual(tb, x);
        squash(x, hist[i]);
      } else if (slot >= 0 && p0 + (tb - s0) >= 0) {
        load_f<V>(tails + ((size_t)slot * K1 + (tb - s0 + K1)) * C + c, hist[i]);
      }
    }
  };
  for (int t = t0; t < t1; ++t) {
    if (TAIL > 0 && t >= s1) enter_run(t);
    float x[V], h[V], y[V];
    residual(t, x);
    if (branch != nullptr) store_act<V>(r_out + (size_t)t * C + c, x);
    squash(x, h);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      float acc = h[e];
#pragma unroll
      for (int i = 0; i < TAIL; ++i) acc = fmaf(cw[i][e], hist[i][e], acc);
      y[e] = fmaf(cw[TAIL][e], h[e], acc);
    }
    store_act<V>(out + (size_t)t * C + c, y);
#pragma unroll
    for (int e = 0; e < V; ++e) {
#pragma unroll
      for (int i = 0; i + 1 < TAIL; ++i) hist[i][e] = hist[i + 1][e];
      if (TAIL > 0) hist[TAIL > 0 ? TAIL - 1 : 0][e] = h[e];
    }
    if (TAIL > 0 && t == s1 - 1 && slot >= 0 && s0 >= t0) {
#pragma unroll
      for (int i = 0; i < TAIL; ++i)
        if (i >= TAIL - K1)
          store_act<V>(tails + ((size_t)slot * K1 + (i - (TAIL - K1))) * C + c, hist[i]);
    }
  }
}

// grid (n_seq, channel blocks): tails of runs that cross a span's border, from
// the updated residual. One thread owns a channel's tail and moves it towards
// the front, so a run shorter than the tail shifts it safely.
__global__ void dyt_tail_kernel(float* __restrict__ tails, const float* __restrict__ r,
                                DytParams pre, const int* __restrict__ start_loc,
                                const int* __restrict__ slots,
                                const int* __restrict__ positions, int C, int K1,
                                int span) {
  const int s = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  const int slot = slots[s], s0 = start_loc[s], n = start_loc[s + 1] - s0;
  if (c >= C || slot < 0 || n <= 0 || s0 / span == (s0 + n - 1) / span) return;
  const int p0 = positions[s0];
  const float al = pre.alpha[0], w = pre.w[c], b = pre.b[c];
  float* tail = tails + (size_t)slot * K1 * C + c;
  for (int i = 0; i < K1; ++i) {
    const int u = n - K1 + i;  // place in the run; negative: carried
    float v = 0.f;
    if (u >= 0) v = fmaf(tanh_f(al * r[(size_t)(s0 + u) * C + c]), w, b);
    else if (p0 + u >= 0) v = tail[(size_t)(i + n) * C];
    tail[(size_t)i * C] = v;
  }
}

}  // namespace

void add_dyt_conv(torch::Tensor out, torch::Tensor new_residual,
                  c10::optional<torch::Tensor> branch,
                  c10::optional<torch::Tensor> post_alpha,
                  c10::optional<torch::Tensor> post_w,
                  c10::optional<torch::Tensor> post_b, torch::Tensor residual,
                  torch::Tensor alpha, torch::Tensor w, torch::Tensor b,
                  c10::optional<torch::Tensor> conv_w,
                  c10::optional<torch::Tensor> tails, torch::Tensor start_loc,
                  torch::Tensor slots, torch::Tensor token_seq,
                  torch::Tensor positions, int64_t max_len) {
  check_f32(residual, "residual");
  check_f32(new_residual, "new_residual");
  check_f32(alpha, "alpha");
  check_f32(w, "w");
  check_f32(b, "b");
  check_i32(start_loc, "start_loc");
  check_i32(slots, "slots");
  check_i32(token_seq, "token_seq");
  check_i32(positions, "positions");
  TORCH_CHECK(residual.dim() == 2 && out.is_cuda() && out.is_contiguous() &&
              out.sizes() == residual.sizes() && new_residual.sizes() == residual.sizes());
  const int T = residual.size(0), C = residual.size(1), n_seq = slots.numel();
  TORCH_CHECK(alpha.numel() == 1 && w.numel() == C && b.numel() == C);
  TORCH_CHECK(start_loc.numel() == n_seq + 1 && token_seq.numel() == T &&
              positions.numel() == T && max_len >= 1);
  TORCH_CHECK(branch.has_value() == post_alpha.has_value() &&
              branch.has_value() == post_w.has_value() &&
              branch.has_value() == post_b.has_value());
  bool wide = false;
  DytParams post{nullptr, nullptr, nullptr};
  const void* bp = nullptr;
  if (branch.has_value()) {
    check_f32(*post_alpha, "post_alpha");
    check_f32(*post_w, "post_w");
    check_f32(*post_b, "post_b");
    TORCH_CHECK(post_alpha->numel() == 1 && post_w->numel() == C && post_b->numel() == C);
    TORCH_CHECK(branch->is_cuda() && branch->is_contiguous() &&
                branch->sizes() == residual.sizes());
    // spans read the tokens ahead of them from the old residual
    TORCH_CHECK(new_residual.data_ptr() != residual.data_ptr(),
                "the updated residual needs a buffer of its own");
    wide = branch->scalar_type() == torch::kFloat32;
    TORCH_CHECK(wide || branch->scalar_type() == out.scalar_type(),
                "branch must be fp32 or the output's dtype");
    post = DytParams{(const float*)post_alpha->data_ptr(), (const float*)post_w->data_ptr(),
                     (const float*)post_b->data_ptr()};
    bp = branch->data_ptr();
  }
  int K1 = 0;
  const float* cwp = nullptr;
  float* tp = nullptr;
  TORCH_CHECK(conv_w.has_value() == tails.has_value());
  if (conv_w.has_value()) {
    check_f32(*conv_w, "conv_w");
    check_f32(*tails, "tails");
    TORCH_CHECK(conv_w->dim() == 2 && conv_w->size(0) == C && conv_w->size(1) >= 1);
    K1 = conv_w->size(1) - 1;
    TORCH_CHECK(K1 <= kMaxConvTail, "at most 16 taps");
    TORCH_CHECK(tails->dim() == 3 && tails->size(1) == K1 && tails->size(2) == C);
    cwp = (const float*)conv_w->data_ptr();
    tp = (float*)tails->data_ptr();
  }
  if (T == 0 || n_seq == 0) return;
  const DytParams pre{(const float*)alpha.data_ptr(), (const float*)w.data_ptr(),
                      (const float*)b.data_ptr()};
  // decode: one token a thread; prompts: long spans repeat fewer inputs, short
  // ones make more blocks
  const int span = max_len == 1 ? 1 : T >= 4096 ? 16 : T >= 512 ? 8 : 4;
  auto al16 = [](const void* p) { return ((size_t)p) % 16 == 0; };
  const bool vec = C % 4 == 0 && al16(out.data_ptr()) && al16(residual.data_ptr()) &&
                   al16(new_residual.data_ptr()) && al16(bp) && al16(pre.w) &&
                   al16(pre.b) && al16(post.w) && al16(post.b) && al16(tp);
  const int V = vec ? 4 : 1;
  const dim3 grid((T + span - 1) / span, (C + 128 * V - 1) / (128 * V));
  TORCH_CHECK(grid.y <= 65535);
  SEQ_DISPATCH_ACT(out, {
    auto go = [&](auto kern, auto* branch_ptr) {
      hipLaunchKernelGGL(kern, grid, dim3(128), 0, SEQ_STREAM(), (act_t*)out.data_ptr(),
                         (float*)new_residual.data_ptr(), branch_ptr, post,
                         (const float*)residual.data_ptr(), pre, cwp, tp,
                         (const int*)start_loc.data_ptr(), (const int*)slots.data_ptr(),
                         (const int*)token_seq.data_ptr(),
                         (const int*)positions.data_ptr(), T, C, K1, span);
    };
    auto by_tail = [&](auto* branch_ptr) {
      using B = std::remove_const_t<std::remove_pointer_t<decltype(branch_ptr)>>;
      if (vec && K1 == 0) go(add_dyt_conv_kernel<act_t, B, 4, 0>, branch_ptr);
      else if (vec && K1 <= 3) go(add_dyt_conv_kernel<act_t, B, 4, 3>, branch_ptr);
      else if (vec && K1 <= 7) go(add_dyt_conv_kernel<act_t, B, 4, 7>, branch_ptr);
      else if (vec) go(add_dyt_conv_kernel<act_t, B, 4, 15>, branch_ptr);
      else if (K1 <= 3) go(add_dyt_conv_kernel<act_t, B, 1, 3>, branch_ptr);
      else go(add_dyt_conv_kernel<act_t, B, 1, 15>, branch_ptr);
    };
    if (wide) by_tail((const float*)bp);
    else by_tail((const act_t*)bp);
  });
  SEQ_CHECK_LAUNCH();
  if (K1 > 0 && max_len > 1) {
    hipLaunchKernelGGL(dyt_tail_kernel, dim3(n_seq, (C + 255) / 256), dim3(256), 0,
                       SEQ_STREAM(), tp, (const float*)new_residual.data_ptr(), pre,
                       (const int*)start_loc.data_ptr(), (const int*)slots.data_ptr(),
                       (const int*)positions.data_ptr(), C, K1, span);
    SEQ_CHECK_LAUNCH();
  }
}
