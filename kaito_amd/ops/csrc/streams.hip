// Hyper-connected residual streams: the stack carries S copies of the
// residual row, x [T, S, H] in f32. A sub-layer reads one weighted sum of
// them and writes back through a matrix:
//
//   u    = sum_s in[s] * x_s                   h = rms(u) * w
//   x_t <- sum_s mix[s, t] * x_s + out[t] * y  (all t from the old streams)
//
// stream_mix_norm fuses one sub-layer's write with the next one's read: a
// row's streams are loaded once, mixed, stored, summed and normed. After
// the last sub-layer it emits the plain weighted sum (no norm, and the
// streams need not be stored). stream_embed opens the stack: table row, RMS
// norm, S equal copies, and the first sub-layer's input.
//
// One workgroup per row. Up to 4 streams and rows of up to 8192 stay in
// registers between the passes (float4 per lane); other sizes take a
// kernel with the thread's old streams in LDS. Norm weights are one number
// per coordinate or a single number for all.
#include "mix_common.h"
#include <type_traits>

namespace kaito {

namespace {

template <int S, int NV, typename T, typename TO>
__global__ __launch_bounds__(512) void stream_mix_norm_kernel(
    float* __restrict__ x, TO* __restrict__ h_out, const T* __restrict__ y,
    const int64_t y_s0, const float* __restrict__ mix,
    const float* __restrict__ w_out, const float* __restrict__ w_in,
    const float* __restrict__ w, const int w_step, const int H,
    const float eps, const bool write_x) {
  __shared__ float red[16];
  const int64_t row = blockIdx.x;
  float* xr = x + row * S * H;
  const T* yr = y + row * y_s0;
  const int nvec = H / 4;
  float m[S][S], wo[S], wi[S];
#pragma unroll
  for (int s = 0; s < S; s++) {
    wo[s] = w_out[s];
    wi[s] = w_in[s];
#pragma unroll
    for (int t = 0; t < S; t++) m[s][t] = mix[s * S + t];
  }
  float4_t xv[NV][S], yv[NV], u[NV];
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = min((int)(threadIdx.x + n * blockDim.x), nvec - 1) * 4;
    yv[n] = act_ld4(yr + i);
#pragma unroll
    for (int s = 0; s < S; s++) xv[n][s] = act_ld4(xr + s * H + i);
  }
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int v = threadIdx.x + n * blockDim.x;
    const bool live = v < nvec;
#pragma unroll
    for (int e = 0; e < 4; e++) {
      float nx[S], a = 0.f;
#pragma unroll
      for (int t = 0; t < S; t++) {
        float acc = wo[t] * yv[n][e];
#pragma unroll
        for (int s = 0; s < S; s++) acc += m[s][t] * xv[n][s][e];
        nx[t] = acc;
        a += wi[t] * acc;
      }
#pragma unroll
      for (int t = 0; t < S; t++) xv[n][t][e] = nx[t];
      u[n][e] = a;
      ss += live ? a * a : 0.f;
    }
    if (live && write_x) {
#pragma unroll
      for (int t = 0; t < S; t++) act_st4(xr + t * H + v * 4, xv[n][t]);
    }
  }
  float inv = 1.0f;
  if (w != nullptr) {
    ss = block_reduce_sum(ss, red);
    inv = 1.0f / sqrtf(ss / (float)H + eps);
  }
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int v = threadIdx.x + n * blockDim.x;
    if (v >= nvec) continue;
    float4_t o = u[n];
    if (w != nullptr) {
#pragma unroll
      for (int e = 0; e < 4; e++) o[e] *= inv * w[(v * 4 + e) * w_step];
    }
    act_st4(h_out + row * H + v * 4, o);
  }
}

// any S and H: the thread's old stream values wait in LDS while the new
// ones are formed; the norm pass re-reads the entries the thread stored
template <typename T, typename TO>
__global__ void stream_mix_norm_any_kernel(
    float* __restrict__ x, TO* __restrict__ h_out, const T* __restrict__ y,
    const int64_t y_s0, const float* __restrict__ mix,
    const float* __restrict__ w_out, const float* __restrict__ w_in,
    const float* __restrict__ w, const int w_step, const int S, const int H,
    const float eps, const bool write_x) {
  extern __shared__ float old[];            // [S][blockDim]
  __shared__ float red[16];
  const int64_t row = blockIdx.x;
  float* xr = x + row * S * H;
  const T* yr = y + row * y_s0;
  const int nt = blockDim.x, tid = threadIdx.x;
  float ss = 0.f;
  for (int i = tid; i < H; i += nt) {
    for (int s = 0; s < S; s++) old[s * nt + tid] = xr[(int64_t)s * H + i];
    const float yi = act_ld(yr + i);
    float u = 0.f;
    for (int t = 0; t < S; t++) {
      float acc = w_out[t] * yi;
      for (int s = 0; s < S; s++) acc += mix[s * S + t] * old[s * nt + tid];
      if (write_x) xr[(int64_t)t * H + i] = acc;
      u += w_in[t] * acc;
    }
    if (w == nullptr) act_st(h_out + row * H + i, u);
    ss += u * u;
  }
  if (w == nullptr) return;
  ss = block_reduce_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)H + eps);
  for (int i = tid; i < H; i += nt) {
    float u = 0.f;
    for (int t = 0; t < S; t++) u += w_in[t] * xr[(int64_t)t * H + i];
    act_st(h_out + row * H + i, u * inv * w[i * w_step]);
  }
}

template <int NV, typename T>
__global__ __launch_bounds__(512) void stream_embed_wide_kernel(
    float* __restrict__ x, T* __restrict__ h_out,
    const int64_t* __restrict__ ids, const T* __restrict__ table,
    const float* __restrict__ g, const int g_step,
    const float* __restrict__ w_in, const float* __restrict__ w,
    const int w_step, const int vocab, const int S, const int H,
    const float eps) {
  __shared__ float red[16];
  const int64_t row = blockIdx.x;
  const int64_t id = ids[row];
  const bool ok = id >= 0 && id < vocab;    // other ids: a row of zeros
  const T* src = table + (ok ? id : 0) * H;
  float* xr = x + row * S * H;
  const int nvec = H / 4;
  float cin = 0.f;
  for (int s = 0; s < S; s++) cin += w_in[s];
  float4_t v[NV];
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    v[n] = i < nvec && ok ? act_ld4(src + i * 4)
                          : float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; e++) ss += v[n][e] * v[n][e];
  }
  ss = block_reduce_sum(ss, red);
  __syncthreads();                          // red[] is used again below
  const float inv = 1.0f / sqrtf(ss / (float)H + eps);
  float su = 0.f;
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    if (i >= nvec) continue;
#pragma unroll
    for (int e = 0; e < 4; e++) {
      v[n][e] *= inv * g[(i * 4 + e) * g_step];
      const float u = cin * v[n][e];
      su += u * u;
    }
    for (int s = 0; s < S; s++) act_st4(xr + (int64_t)s * H + i * 4, v[n]);
  }
  su = block_reduce_sum(su, red);
  const float inv_u = 1.0f / sqrtf(su / (float)H + eps);
#pragma unroll
  for (int n = 0; n < NV; n++) {
    const int i = threadIdx.x + n * blockDim.x;
    if (i >= nvec) continue;
    float4_t o;
#pragma unroll
    for (int e = 0; e < 4; e++)
      o[e] = cin * v[n][e] * inv_u * w[(i * 4 + e) * w_step];
    act_st4(h_out + row * H + i * 4, o);
  }
}

template <typename T>
__global__ void stream_embed_kernel(
    float* __restrict__ x, T* __restrict__ h_out,
    const int64_t* __restrict__ ids, const T* __restrict__ table,
    const float* __restrict__ g, const int g_step,
    const float* __restrict__ w_in, const float* __restrict__ w,
    const int w_step, const int vocab, const int S, const int H,
    const float eps) {
  __shared__ float red[16];
  const int64_t row = blockIdx.x;
  const int64_t id = ids[row];
  const bool ok = id >= 0 && id < vocab;    // other ids: a row of zeros
  const T* src = table + (ok ? id : 0) * H;
  float* xr = x + row * S * H;
  float cin = 0.f;
  for (int s = 0; s < S; s++) cin += w_in[s];
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float v = ok ? act_ld(src + i) : 0.f;
    ss += v * v;
  }
  ss = block_reduce_sum(ss, red);
  __syncthreads();                          // red[] is used again below
  const float inv = 1.0f / sqrtf(ss / (float)H + eps);
  float su = 0.f;
  for (int i = threadIdx.x; i < H; i += blockDim.x) {
    const float v = (ok ? act_ld(src + i) : 0.f) * inv * g[i * g_step];
    for (int s = 0; s < S; s++) xr[(int64_t)s * H + i] = v;
    const float u = cin * v;
    su += u * u;
  }
  su = block_reduce_sum(su, red);
  const float inv_u = 1.0f / sqrtf(su / (float)H + eps);
  for (int i = threadIdx.x; i < H; i += blockDim.x)
    act_st(h_out + row * H + i, cin * xr[i] * inv_u * w[i * w_step]);
}

int row_threads(int H) { return H >= 1024 ? 256 : (H >= 256 ? 128 : 64); }

void check_weight(const at::Tensor& w, int H) {
  KAITO_CHECK_F32(w);
  TORCH_CHECK(w.numel() == 1 || w.numel() == H);
}

int weight_step(const at::Tensor& w, int H) {
  return w.numel() == H ? 1 : 0;            // H = 1: index 0 either way
}

}  // namespace

void stream_mix_norm(at::Tensor x, at::Tensor h_out, at::Tensor y,
                     at::Tensor mix, at::Tensor w_out, at::Tensor w_in,
                     at::Tensor w, double eps, bool write_x) {
  KAITO_CHECK_F32(x);
  TORCH_CHECK(x.dim() == 3);
  const int T = x.size(0), S = x.size(1), H = x.size(2);
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.stride(1) == 1 &&
              y.size(0) == T && y.size(1) == H && is_act_dtype(y));
  TORCH_CHECK(h_out.is_cuda() && h_out.is_contiguous() && h_out.dim() == 2 &&
              h_out.size(0) == T && h_out.size(1) == H &&
              is_act_dtype(h_out));
  KAITO_CHECK_F32(mix); KAITO_CHECK_F32(w_out); KAITO_CHECK_F32(w_in);
  TORCH_CHECK(mix.numel() == (int64_t)S * S && w_out.numel() == S &&
              w_in.numel() == S);
  const bool norm = w.numel() > 0;
  if (norm) check_weight(w, H);
  TORCH_CHECK(write_x || !norm, "a norm follows stored streams only");
  if (T == 0 || H == 0) return;
  const float* wp = norm ? w.data_ptr<float>() : nullptr;
  const int step = norm ? weight_step(w, H) : 0;
  auto stream = at::hip::getCurrentHIPStream();
  KAITO_DISPATCH_ACT(y, {
    using in_t = act_t;
    KAITO_DISPATCH_ACT(h_out, {
      using out_t = act_t;
      const bool wide = H % 4 == 0 && H <= 8192 && S <= 4 &&
          y.stride(0) % 4 == 0 &&
          (uintptr_t)y.data_ptr() % (4 * sizeof(in_t)) == 0 &&
          (uintptr_t)h_out.data_ptr() % (4 * sizeof(out_t)) == 0;
      if (wide) {
        const int nvec = H / 4;
        const int threads = std::min(512, (nvec + 63) / 64 * 64);
        const int nv = (nvec + threads - 1) / threads;
        auto launch = [&](auto s_c, auto nv_c) {
          hipLaunchKernelGGL((stream_mix_norm_kernel<decltype(s_c)::value,
                                  decltype(nv_c)::value, in_t, out_t>),
              dim3(T), dim3(threads), 0, stream, x.data_ptr<float>(),
              (out_t*)h_out.data_ptr(), (const in_t*)y.data_ptr(),
              y.stride(0), mix.data_ptr<float>(), w_out.data_ptr<float>(),
              w_in.data_ptr<float>(), wp, step, H, (float)eps, write_x);
        };
        auto by_nv = [&](auto s_c) {
          if (nv == 1) launch(s_c, std::integral_constant<int, 1>{});
          else if (nv == 2) launch(s_c, std::integral_constant<int, 2>{});
          else launch(s_c, std::integral_constant<int, 4>{});
        };
        if (S == 1) by_nv(std::integral_constant<int, 1>{});
        else if (S == 2) by_nv(std::integral_constant<int, 2>{});
        else if (S == 3) by_nv(std::integral_constant<int, 3>{});
        else by_nv(std::integral_constant<int, 4>{});
      } else {
        int threads = row_threads(H);
        while (threads > 64 && (size_t)S * threads * 4 > 32768) threads >>= 1;
        const size_t lds = (size_t)S * threads * 4;
        TORCH_CHECK(lds <= 65536 - 64, "too many streams: ", S);
        hipLaunchKernelGGL((stream_mix_norm_any_kernel<in_t, out_t>),
            dim3(T), dim3(threads), lds, stream, x.data_ptr<float>(),
            (out_t*)h_out.data_ptr(), (const in_t*)y.data_ptr(), y.stride(0),
            mix.data_ptr<float>(), w_out.data_ptr<float>(),
            w_in.data_ptr<float>(), wp, step, S, H, (float)eps, write_x);
      }
    });
  });
}

void stream_embed(at::Tensor x, at::Tensor h_out, at::Tensor ids,
                  at::Tensor table, at::Tensor g, at::Tensor w_in,
                  at::Tensor w, double eps) {
  KAITO_CHECK_F32(x);
  TORCH_CHECK(x.dim() == 3);
  const int T = x.size(0), S = x.size(1), H = x.size(2);
  TORCH_CHECK(table.is_cuda() && table.is_contiguous() && table.dim() == 2 &&
              table.size(0) > 0 && table.size(1) == H && is_act_dtype(table));
  TORCH_CHECK(h_out.is_cuda() && h_out.is_contiguous() && h_out.dim() == 2 &&
              h_out.size(0) == T && h_out.size(1) == H &&
              h_out.dtype() == table.dtype());
  TORCH_CHECK(ids.is_cuda() && ids.is_contiguous() &&
              ids.dtype() == at::kLong && ids.numel() == T);
  check_weight(g, H);
  check_weight(w, H);
  KAITO_CHECK_F32(w_in);
  TORCH_CHECK(w_in.numel() == S);
  if (T == 0 || H == 0) return;
  auto stream = at::hip::getCurrentHIPStream();
  KAITO_DISPATCH_ACT(table, {
    auto launch = [&](auto kernel, int threads) {
      hipLaunchKernelGGL(kernel, dim3(T), dim3(threads), 0, stream,
          x.data_ptr<float>(), (act_t*)h_out.data_ptr(),
          ids.data_ptr<int64_t>(), (const act_t*)table.data_ptr(),
          g.data_ptr<float>(), weight_step(g, H), w_in.data_ptr<float>(),
          w.data_ptr<float>(), weight_step(w, H), (int)table.size(0), S, H,
          (float)eps);
    };
    if (H % 4 == 0 && H <= 8192 &&
        (uintptr_t)table.data_ptr() % (4 * sizeof(act_t)) == 0 &&
        (uintptr_t)h_out.data_ptr() % (4 * sizeof(act_t)) == 0) {
      const int threads = std::min(512, (H / 4 + 63) / 64 * 64);
      if (H / 4 <= threads)
        launch(stream_embed_wide_kernel<1, act_t>, threads);
      else
        launch(stream_embed_wide_kernel<4, act_t>, threads);
    } else {
      launch(stream_embed_kernel<act_t>, row_threads(H));
    }
  });
}

}  // namespace kaito

TORCH_LIBRARY_FRAGMENT(kaito, m) {
  m.def("stream_mix_norm(Tensor(a!) x, Tensor(b!) h_out, Tensor y, Tensor mix, Tensor w_out, Tensor w_in, Tensor w, float eps, bool write_x) -> ()");
  m.def("stream_embed(Tensor(a!) x, Tensor(b!) h_out, Tensor ids, Tensor table, Tensor g, Tensor w_in, Tensor w, float eps) -> ()");
}
TORCH_LIBRARY_IMPL(kaito, CUDA, m) {
  m.impl("stream_mix_norm", &kaito::stream_mix_norm);
  m.impl("stream_embed", &kaito::stream_embed);
}
