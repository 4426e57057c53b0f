// Expert choice for routed feed-forwards, in two launches.
//
//   moe_route: one wave per token. s = softmax(logits); choice = s +
//     correction (none given: s); the outputs form `groups` equal groups of neighbours, a
//     group scores its largest choice, only the `keep` best groups stay
//     eligible; the `top` largest eligible choices are taken (ties: lower
//     index). Weights are the taken s (without the correction), divided by
//     their sum + 1e-20 when `renorm`, times `scale`. Outputs with index >=
//     n_real are identity experts: their weights are also summed per token.
//   moe_sort: one workgroup. Counting sort of the (token, expert) pairs by
//     expert: token and weight of every sorted row, exclusive offsets.
//
// An output's place in the row lives in lane e % 64, register e / 64.
#include "mix_common.h"
#include <type_traits>

namespace kaito {

namespace {

constexpr int ROUTE_MAX = 1024;      // router outputs

// largest value over the wave, ties to the lower index
KAITO_DEV void wave_argmax(float& v, int& i) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    const float ov = __shfl_xor(v, off, 64);
    const int oi = __shfl_xor(i, off, 64);
    if (ov > v || (ov == v && oi < i)) { v = ov; i = oi; }
  }
}

template <int NPL>
__global__ __launch_bounds__(256) void moe_route_kernel(
    int* __restrict__ topi, float* __restrict__ topw,
    float* __restrict__ w_id, const float* __restrict__ logits,
    const float* __restrict__ correction, const int T, const int N,
    const int n_real, const int top, const int groups, const int keep,
    const bool renorm, const float scale) {
  const int lane = threadIdx.x & 63;
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= T) return;                       // whole waves; no barriers below
  const float* row = logits + (int64_t)t * N;
  float s[NPL], ch[NPL];
  float mx = -INFINITY;
#pragma unroll
  for (int r = 0; r < NPL; r++) {
    const int e = r * 64 + lane;
    s[r] = e < N ? row[e] : -INFINITY;
    mx = fmaxf(mx, s[r]);
  }
  mx = wave_reduce_max(mx);
  float sum = 0.f;
#pragma unroll
  for (int r = 0; r < NPL; r++) {
    s[r] = r * 64 + lane < N ? expf(s[r] - mx) : 0.f;
    sum += s[r];
  }
  sum = wave_reduce_sum(sum);
#pragma unroll
  for (int r = 0; r < NPL; r++) {
    const int e = r * 64 + lane;
    s[r] = s[r] / sum;
    ch[r] = e < N ? s[r] + (correction ? correction[e] : 0.f) : -INFINITY;
  }
  if (groups > 1) {
    const int n = N / groups;
    float mine = -INFINITY;                 // lane g: group g's score
    for (int g = 0; g < groups; g++) {
      float m = -INFINITY;
#pragma unroll
      for (int r = 0; r < NPL; r++) {
        const int e = r * 64 + lane;
        if (e >= g * n && e < (g + 1) * n) m = fmaxf(m, ch[r]);
      }
      m = wave_reduce_max(m);
      if (lane == g) mine = m;
    }
    unsigned long long kept = 0;
    for (int k = 0; k < keep; k++) {
      float v = mine;
      int i = lane;
      wave_argmax(v, i);
      kept |= 1ull << i;
      if (lane == i) mine = -INFINITY;
    }
#pragma unroll
    for (int r = 0; r < NPL; r++) {
      const int e = r * 64 + lane;
      if (e < N && !((kept >> (e / n)) & 1)) ch[r] = -INFINITY;
    }
  }
  float wsum = 0.f, mine = 0.f;             // lane k: k-th taken weight
  int mine_i = 0;
  for (int k = 0; k < top; k++) {
    float v = -INFINITY;
    int i = min(lane, N - 1);
#pragma unroll
    for (int r = 0; r < NPL; r++)
      if (ch[r] > v) { v = ch[r]; i = r * 64 + lane; }
    wave_argmax(v, i);
    float sv = 0.f;
#pragma unroll
    for (int r = 0; r < NPL; r++) {
      const float b = __shfl(s[r], i & 63, 64);
      if (r == (i >> 6)) sv = b;
      if (r * 64 + lane == i) ch[r] = -INFINITY;
    }
    wsum += sv;
    if (lane == k) { mine = sv; mine_i = i; }
  }
  const float f = renorm ? scale / (wsum + 1e-20f) : scale;
  mine *= f;
  if (lane < top) {
    topi[(int64_t)t * top + lane] = mine_i;
    topw[(int64_t)t * top + lane] = mine;
  }
  const float idw = wave_reduce_sum(lane < top && mine_i >= n_real ? mine
                                                                   : 0.f);
  if (lane == 0) w_id[t] = idw;
}

__global__ __launch_bounds__(1024) void moe_sort_kernel(
    int* __restrict__ sorted_tok, float* __restrict__ gates,
    int* __restrict__ offsets, const int* __restrict__ topi,
    const float* __restrict__ topw, const int TK, const int top,
    const int N) {
  __shared__ int scan[ROUTE_MAX];
  const int tid = threadIdx.x;
  scan[tid] = 0;
  __syncthreads();
  for (int i = tid; i < TK; i += 1024) atomicAdd(&scan[topi[i]], 1);
  __syncthreads();
  const int count = scan[tid];
  for (int off = 1; off < N; off <<= 1) {   // inclusive scan
    const int add = tid >= off ? scan[tid - off] : 0;
    __syncthreads();
    scan[tid] += add;
    __syncthreads();
  }
  if (tid == 0) offsets[0] = 0;
  if (tid < N) offsets[tid + 1] = scan[tid];
  __syncthreads();
  scan[tid] -= count;                       // next free row of the expert
  __syncthreads();
  for (int i = tid; i < TK; i += 1024) {
    const int at = atomicAdd(&scan[topi[i]], 1);
    sorted_tok[at] = i / top;
    gates[at] = topw[i];
  }
}

}  // namespace

void moe_route(at::Tensor topi, at::Tensor topw, at::Tensor w_id,
               at::Tensor logits, at::Tensor correction, int64_t n_real,
               int64_t groups, int64_t keep, bool renorm, double scale) {
  KAITO_CHECK_F32(logits);
  const bool corr = correction.numel() > 0;
  if (corr) KAITO_CHECK_F32(correction);
  KAITO_CHECK_I32(topi); KAITO_CHECK_F32(topw); KAITO_CHECK_F32(w_id);
  TORCH_CHECK(logits.dim() == 2 && topi.dim() == 2);
  const int T = logits.size(0), N = logits.size(1), top = topi.size(1);
  TORCH_CHECK(topi.size(0) == T && topw.sizes() == topi.sizes() &&
              w_id.numel() == T && (!corr || correction.numel() == N));
  TORCH_CHECK(N >= 1 && N <= ROUTE_MAX && top >= 1 && top <= 64 && top <= N);
  TORCH_CHECK(groups >= 1 && groups <= 64 && N % groups == 0 && keep >= 1 &&
              keep <= groups);
  if (T == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  auto launch = [&](auto npl) {
    hipLaunchKernelGGL((moe_route_kernel<decltype(npl)::value>),
        dim3((T + 3) / 4), dim3(256), 0, stream, topi.data_ptr<int>(),
        topw.data_ptr<float>(), w_id.data_ptr<float>(),
        logits.data_ptr<float>(),
        corr ? correction.data_ptr<float>() : nullptr, T, N,
        (int)n_real, top, (int)groups, (int)keep, renorm, (float)scale);
  };
  if (N <= 64) launch(std::integral_constant<int, 1>{});
  else if (N <= 128) launch(std::integral_constant<int, 2>{});
  else if (N <= 256) launch(std::integral_constant<int, 4>{});
  else launch(std::integral_constant<int, 16>{});
}

void moe_sort(at::Tensor sorted_tok, at::Tensor gates, at::Tensor offsets,
              at::Tensor topi, at::Tensor topw) {
  KAITO_CHECK_I32(topi); KAITO_CHECK_F32(topw);
  KAITO_CHECK_I32(sorted_tok); KAITO_CHECK_F32(gates);
  KAITO_CHECK_I32(offsets);
  TORCH_CHECK(topi.dim() == 2 && topw.sizes() == topi.sizes());
  TORCH_CHECK(topi.numel() < (1ll << 31));
  const int TK = topi.numel(), top = topi.size(1);
  const int N = offsets.numel() - 1;
  TORCH_CHECK(sorted_tok.numel() == TK && gates.numel() == TK && N >= 1 &&
              N <= ROUTE_MAX);
  auto stream = at::hip::getCurrentHIPStream();
  hipLaunchKernelGGL(moe_sort_kernel, dim3(1), dim3(1024), 0, stream,
      sorted_tok.data_ptr<int>(), gates.data_ptr<float>(),
      offsets.data_ptr<int>(), topi.data_ptr<int>(), topw.data_ptr<float>(),
      TK, top, N);
}

}  // namespace kaito

TORCH_LIBRARY_FRAGMENT(kaito, m) {
  m.def("moe_route(Tensor(a!) topi, Tensor(b!) topw, Tensor(c!) w_id, Tensor logits, Tensor correction, int n_real, int groups, int keep, bool renorm, float scale) -> ()");
  m.def("moe_sort(Tensor(a!) sorted_tok, Tensor(b!) gates, Tensor(c!) offsets, Tensor topi, Tensor topw) -> ()");
}
TORCH_LIBRARY_IMPL(kaito, CUDA, m) {
  m.impl("moe_route", &kaito::moe_route);
  m.impl("moe_sort", &kaito::moe_sort);
}
