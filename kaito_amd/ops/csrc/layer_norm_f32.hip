// Layer norms (weight and bias, f32) around an f32 residual stream:
//
//   ln(v) = (v - mean) / sqrt(mean((v - mean)^2) + eps) * w + b
//
//   layer_norm_cast:         ln(x) for f32 or bf16 rows -> f32 or bf16
//   embed_layer_norm:        x32 = table[id] * scale, h = ln(x32)
//   sandwich_norm_residual:  x32 += ln_b(y + y2)      (in place, f32)
//                            h    = ln_a(x32)          (next input)
//
// One workgroup per row. The variance is taken around the mean (two passes
// over the row, which waits in registers as float4; rows too long for that,
// or not in 16-byte steps, are read again instead: a thread only re-reads
// what it wrote itself).
#include "mix_common.h"
#include <type_traits>

namespace kaito {

namespace {

// mean and 1/sqrt(variance + eps) of a row held as v[NV] (nvec float4 in
// all, lanes past the end hold zeros)
template <int NV>
KAITO_DEV void row_stats(const float4_t (&v)[NV], const int nvec,
                         const int H, const float eps, float (&red)[2][16],
                         float& mean, float& inv) {
  float s = 0.f;
#pragma unroll
  for (int n = 0; n < NV; n++)
#pragma unroll
    for (int e = 0; e < 4; e++) s += v[n][e];
  mean = block_reduce_sum(s, red[0]) / (float)H;
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < NV; n++) {
    if ((int)threadIdx.x + n * (int)blockDim.x >= nvec) continue;
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const float c = v[n][e] - mean;
      ss += c * c;
    }
  }
  inv = 1.0f / sqrtf(block_reduce_sum(ss, red[1]) / (float)H + eps);
}

KAITO_DEV float4_t ln4(const float4_t v, const float mean, const float inv,
                       const float4_t w, const float4_t b) {
  float4_t o;
#pragma unroll
  for (int e = 0; e < 4; e++) o[e] = (v[e] - mean) * inv * w[e] + b[e];
  return o;
}

KAITO_DEV float4_t ld4(const float* p) {
  return *reinterpret_cast<const float4_t*>(p);
}

template <int NV, typename TI, typename TO>
__global__ __launch_bounds__(512) void layer_norm_wide_kernel(
    TO* __restrict__ out, const TI* __restrict__ x,
    const float* __restrict__ w, const float* __restrict__ b, const int H,
    const float eps) {
  __shared__ float red[2][16];
  const int64_t row = blockIdx.x;
  const int nvec = H / 4;
  float4_t v[NV];
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    v[n] = i < nvec ? act_ld4(x + row * H + i * 4)
                    : float4_t{0.f, 0.f, 0.f, 0.f};
  }
  float mean, inv;
  row_stats<NV>(v, nvec, H, eps, red, mean, inv);
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    if (i < nvec)
      act_st4(out + row * H + i * 4,
              ln4(v[n], mean, inv, ld4(w + i * 4), ld4(b + i * 4)));
  }
}

template <int NV, typename T>
__global__ __launch_bounds__(512) void embed_layer_norm_wide_kernel(
    float* __restrict__ x32, T* __restrict__ h,
    const int64_t* __restrict__ ids, const T* __restrict__ table,
    const float scale, const float* __restrict__ w,
    const float* __restrict__ b, const int vocab, const int H,
    const float eps) {
  __shared__ float red[2][16];
  const int64_t row = blockIdx.x;
  const int64_t id = ids[row];
  const bool ok = id >= 0 && id < vocab;    // other ids: a row of zeros
  const T* src = table + (ok ? id : 0) * H;
  const int nvec = H / 4;
  float4_t v[NV];
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    v[n] = i < nvec && ok ? act_ld4(src + i * 4)
                          : float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; e++) v[n][e] *= scale;
    if (i < nvec) act_st4(x32 + row * H + i * 4, v[n]);
  }
  float mean, inv;
  row_stats<NV>(v, nvec, H, eps, red, mean, inv);
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    if (i < nvec)
      act_st4(h + row * H + i * 4,
              ln4(v[n], mean, inv, ld4(w + i * 4), ld4(b + i * 4)));
  }
}

// y2 is in the activation dtype of the output; wn null = no next norm
template <int NV, typename TY, typename TO>
__global__ __launch_bounds__(512) void sandwich_norm_wide_kernel(
    float* __restrict__ x32, TO* __restrict__ h, const TY* __restrict__ y,
    const int64_t y_s0, const TO* __restrict__ y2, const int64_t y2_s0,
    const float* __restrict__ w, const float* __restrict__ b,
    const float* __restrict__ wn, const float* __restrict__ bn, const int H,
    const float eps) {
  __shared__ float red[2][2][16];
  const int64_t row = blockIdx.x;
  const int nvec = H / 4;
  float* xr = x32 + row * H;
  float4_t v[NV], x[NV];
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    const bool in = i < nvec;
    const float4_t zero{0.f, 0.f, 0.f, 0.f};
    v[n] = in ? act_ld4(y + row * y_s0 + i * 4) : zero;
    x[n] = in ? ld4(xr + i * 4) : zero;
    if (y2 != nullptr && in) v[n] += act_ld4(y2 + row * y2_s0 + i * 4);
  }
  float mean, inv;
  row_stats<NV>(v, nvec, H, eps, red[0], mean, inv);
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    if (i >= nvec) continue;
    x[n] += ln4(v[n], mean, inv, ld4(w + i * 4), ld4(b + i * 4));
    act_st4(xr + i * 4, x[n]);
  }
  if (wn == nullptr) return;
  row_stats<NV>(x, nvec, H, eps, red[1], mean, inv);
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    if (i < nvec)
      act_st4(h + row * H + i * 4,
              ln4(x[n], mean, inv, ld4(wn + i * 4), ld4(bn + i * 4)));
  }
}

// ---- any row length and alignment ---------------------------------------------

// `at(i)` reads element i of the row
template <typename F>
KAITO_DEV void any_stats(F at, const int H, const float eps,
                         float (&red)[2][16], float& mean, float& inv) {
  float s = 0.f;
  for (int i = threadIdx.x; i < H; i += blockDim.x) s += at(i);
  mean = block_reduce_sum(s, red[0]) / (float)H;
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float c = at(i) - mean;
    ss += c * c;
  }
  inv = 1.0f / sqrtf(block_reduce_sum(ss, red[1]) / (float)H + eps);
}

template <typename TI, typename TO>
__global__ void layer_norm_any_kernel(TO* __restrict__ out,
                                      const TI* __restrict__ x,
                                      const float* __restrict__ w,
                                      const float* __restrict__ b,
                                      const int H, const float eps) {
  __shared__ float red[2][16];
  const int64_t row = blockIdx.x;
  const TI* xr = x + row * H;
  float mean, inv;
  any_stats([&](int i) { return act_ld(xr + i); }, H, eps, red, mean, inv);
  for (int i = threadIdx.x; i < H; i += blockDim.x)
    act_st(out + row * H + i, (act_ld(xr + i) - mean) * inv * w[i] + b[i]);
}

template <typename T>
__global__ void embed_layer_norm_any_kernel(
    float* __restrict__ x32, T* __restrict__ h,
    const int64_t* __restrict__ ids, const T* __restrict__ table,
    const float scale, const float* __restrict__ w,
    const float* __restrict__ b, const int vocab, const int H,
    const float eps) {
  __shared__ float red[2][16];
  const int64_t row = blockIdx.x;
  const int64_t id = ids[row];
  const bool ok = id >= 0 && id < vocab;
  const T* src = table + (ok ? id : 0) * H;
  float* xr = x32 + row * H;
  for (int i = threadIdx.x; i < H; i += blockDim.x)
    xr[i] = ok ? act_ld(src + i) * scale : 0.f;
  float mean, inv;
  any_stats([&](int i) { return xr[i]; }, H, eps, red, mean, inv);
  for (int i = threadIdx.x; i < H; i += blockDim.x)
    act_st(h + row * H + i, (xr[i] - mean) * inv * w[i] + b[i]);
}

template <typename TY, typename TO>
__global__ void sandwich_norm_any_kernel(
    float* __restrict__ x32, TO* __restrict__ h, const TY* __restrict__ y,
    const int64_t y_s0, const TO* __restrict__ y2, const int64_t y2_s0,
    const float* __restrict__ w, const float* __restrict__ b,
    const float* __restrict__ wn, const float* __restrict__ bn, const int H,
    const float eps) {
  __shared__ float red[2][2][16];
  const int64_t row = blockIdx.x;
  float* xr = x32 + row * H;
  auto m = [&](int i) {
    float v = act_ld(y + row * y_s0 + i);
    if (y2 != nullptr) v += act_ld(y2 + row * y2_s0 + i);
    return v;
  };
  float mean, inv;
  any_stats(m, H, eps, red[0], mean, inv);
  for (int i = threadIdx.x; i < H; i += blockDim.x)
    xr[i] += (m(i) - mean) * inv * w[i] + b[i];
  if (wn == nullptr) return;
  any_stats([&](int i) { return xr[i]; }, H, eps, red[1], mean, inv);
  for (int i = threadIdx.x; i < H; i += blockDim.x)
    act_st(h + row * H + i, (xr[i] - mean) * inv * wn[i] + bn[i]);
}

int row_threads(int H) { return H >= 1024 ? 256 : (H >= 256 ? 128 : 64); }

bool aligned4(const at::Tensor& t) {
  return (uintptr_t)t.data_ptr() % (4 * t.element_size()) == 0;
}

void check_norm(const at::Tensor& w, const at::Tensor& b, int H) {
  KAITO_CHECK_F32(w); KAITO_CHECK_F32(b);
  TORCH_CHECK(w.numel() == H && b.numel() == H,
              "layer norm: weight and bias of ", H, " numbers");
}

// float4 per thread of a row of H: threads and the NV that covers it
template <typename F>
void wide_launch(int H, F launch) {
  const int nvec = H / 4;
  const int threads = std::min(512, (nvec + 63) / 64 * 64);
  const int nv = (nvec + threads - 1) / threads;
  if (nv == 1) launch(std::integral_constant<int, 1>{}, threads);
  else if (nv == 2) launch(std::integral_constant<int, 2>{}, threads);
  else launch(std::integral_constant<int, 4>{}, threads);
}

}  // namespace

void layer_norm_cast(at::Tensor out, at::Tensor x, at::Tensor w, at::Tensor b,
                     double eps) {
  TORCH_CHECK(x.is_cuda() && x.is_contiguous() && is_act_dtype(x) &&
              x.dim() == 2 && out.is_cuda() && out.is_contiguous() &&
              is_act_dtype(out) && out.sizes() == x.sizes());
  const int T = x.size(0), H = x.size(1);
  check_norm(w, b, H);
  if (T == 0 || H == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const bool wide = H % 4 == 0 && H <= 8192 && aligned4(x) && aligned4(out) &&
      aligned4(w) && aligned4(b);
  KAITO_DISPATCH_ACT(x, {
    using in_t = act_t;
    KAITO_DISPATCH_ACT(out, {
      using out_t = act_t;
      auto launch = [&](auto kernel, int threads) {
        hipLaunchKernelGGL(kernel, dim3(T), dim3(threads), 0, stream,
            (out_t*)out.data_ptr(), (const in_t*)x.data_ptr(),
            w.data_ptr<float>(), b.data_ptr<float>(), H, (float)eps);
      };
      if (wide)
        wide_launch(H, [&](auto nv, int threads) {
          launch(layer_norm_wide_kernel<decltype(nv)::value, in_t, out_t>,
                 threads);
        });
      else
        launch(layer_norm_any_kernel<in_t, out_t>, row_threads(H));
    });
  });
}

void embed_layer_norm(at::Tensor x32, at::Tensor h, at::Tensor ids,
                      at::Tensor table, double scale, at::Tensor w,
                      at::Tensor b, double eps) {
  KAITO_CHECK_F32(x32);
  TORCH_CHECK(x32.dim() == 2);
  const int T = x32.size(0), H = x32.size(1);
  TORCH_CHECK(table.is_cuda() && table.is_contiguous() && table.dim() == 2 &&
              table.size(0) > 0 && table.size(1) == H && is_act_dtype(table));
  TORCH_CHECK(h.is_cuda() && h.is_contiguous() && h.sizes() == x32.sizes() &&
              h.dtype() == table.dtype());
  TORCH_CHECK(ids.is_cuda() && ids.is_contiguous() &&
              ids.dtype() == at::kLong && ids.numel() == T);
  check_norm(w, b, H);
  if (T == 0 || H == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const bool wide = H % 4 == 0 && H <= 8192 && aligned4(table) &&
      aligned4(x32) && aligned4(h) && aligned4(w) && aligned4(b);
  KAITO_DISPATCH_ACT(table, {
    auto launch = [&](auto kernel, int threads) {
      hipLaunchKernelGGL(kernel, dim3(T), dim3(threads), 0, stream,
          x32.data_ptr<float>(), (act_t*)h.data_ptr(),
          ids.data_ptr<int64_t>(), (const act_t*)table.data_ptr(),
          (float)scale, w.data_ptr<float>(), b.data_ptr<float>(),
          (int)table.size(0), H, (float)eps);
    };
    if (wide)
      wide_launch(H, [&](auto nv, int threads) {
        launch(embed_layer_norm_wide_kernel<decltype(nv)::value, act_t>,
               threads);
      });
    else
      launch(embed_layer_norm_any_kernel<act_t>, row_threads(H));
  });
}

void sandwich_norm_residual(at::Tensor x32, at::Tensor h, at::Tensor y,
                            at::Tensor y2, at::Tensor w, at::Tensor b,
                            at::Tensor w_next, at::Tensor b_next,
                            double eps) {
  KAITO_CHECK_F32(x32);
  TORCH_CHECK(x32.dim() == 2 && y.is_cuda() && y.dim() == 2 &&
              y.stride(1) == 1 && y.sizes() == x32.sizes() &&
              is_act_dtype(y));
  const int T = x32.size(0), H = x32.size(1);
  check_norm(w, b, H);
  const bool next = w_next.numel() > 0, pair = y2.numel() > 0;
  if (next) {
    check_norm(w_next, b_next, H);
    TORCH_CHECK(h.is_cuda() && h.is_contiguous() &&
                h.sizes() == x32.sizes() && is_act_dtype(h) &&
                h.data_ptr() != x32.data_ptr());
  }
  // the second addend decides the activation dtype when no input follows
  const at::Tensor& act = next ? h : (pair ? y2 : y);
  if (pair)
    TORCH_CHECK(y2.is_cuda() && y2.dim() == 2 && y2.stride(1) == 1 &&
                y2.sizes() == x32.sizes() && y2.dtype() == act.dtype());
  if (T == 0 || H == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  const bool wide = H % 4 == 0 && H <= 8192 && y.stride(0) % 4 == 0 &&
      aligned4(y) && aligned4(x32) && aligned4(w) && aligned4(b) &&
      (!pair || (y2.stride(0) % 4 == 0 && aligned4(y2))) &&
      (!next || (aligned4(h) && aligned4(w_next) && aligned4(b_next)));
  KAITO_DISPATCH_ACT(y, {
    using in_t = act_t;
    KAITO_DISPATCH_ACT(act, {
      using out_t = act_t;
      auto launch = [&](auto kernel, int threads) {
        hipLaunchKernelGGL(kernel, dim3(T), dim3(threads), 0, stream,
            x32.data_ptr<float>(), next ? (out_t*)h.data_ptr() : nullptr,
            (const in_t*)y.data_ptr(), y.stride(0),
            pair ? (const out_t*)y2.data_ptr() : nullptr,
            pair ? y2.stride(0) : 0, w.data_ptr<float>(),
            b.data_ptr<float>(), next ? w_next.data_ptr<float>() : nullptr,
            next ? b_next.data_ptr<float>() : nullptr, H, (float)eps);
      };
      if (wide)
        wide_launch(H, [&](auto nv, int threads) {
          launch(sandwich_norm_wide_kernel<decltype(nv)::value, in_t, out_t>,
                 threads);
        });
      else
        launch(sandwich_norm_any_kernel<in_t, out_t>, row_threads(H));
    });
  });
}

}  // namespace kaito

TORCH_LIBRARY_FRAGMENT(kaito, m) {
  m.def("layer_norm_cast(Tensor(a!) out, Tensor x, Tensor w, Tensor b, float eps) -> ()");
  m.def("embed_layer_norm(Tensor(a!) x32, Tensor(b!) h, Tensor ids, Tensor table, float scale, Tensor w, Tensor b, float eps) -> ()");
  m.def("sandwich_norm_residual(Tensor(a!) x32, Tensor(b!) h, Tensor y, Tensor y2, Tensor w, Tensor b, Tensor w_next, Tensor b_next, float eps) -> ()");
}
TORCH_LIBRARY_IMPL(kaito, CUDA, m) {
  m.impl("layer_norm_cast", &kaito::layer_norm_cast);
  m.impl("embed_layer_norm", &kaito::embed_layer_norm);
  m.impl("sandwich_norm_residual", &kaito::sandwich_norm_residual);
}
