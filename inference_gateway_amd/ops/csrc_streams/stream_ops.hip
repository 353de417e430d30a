// Row kernels of a decoder with several residual streams and of its
// mixture of experts (gfx950):
//
//   stream_step       X'_t = sum_b M[b, t] X_b + c_t y   (X [T, B, D] fp32)
//                     out  = rmsnorm(sum_t a_t X'_t) * w
//   moe_scatter_rows  row dst[t, k] of a padded buffer = x[t]
//   moe_combine       out[t] = sum_k w[t, k] y[dst[t, k]]
//                              + sigmoid(g[t]) shared[t]
//
// stream_step is the whole step between two sublayers: the previous
// sublayer's result goes into every stream, the next sublayer's input is
// read off the new streams and normed, one pass over the streams.  Without
// y nothing is updated and the input comes from X itself; X may repeat one
// row for all streams (stream stride 0: the state after the embedding), in
// which case the new streams go to a buffer of their own.
#include "../csrc_hybrid/act_types.h"

namespace igw {

constexpr int ST_BLOCK = 256;

// four consecutive activations
template <typename T>
struct Act4;
template <>
struct Act4<float> {
  static DEVINLINE float4 ld(const float* p) { return *(const float4*)p; }
  static DEVINLINE void st(float* p, float4 v) { *(float4*)p = v; }
};
template <>
struct Act4<uint16_t> {
  static DEVINLINE float4 ld(const uint16_t* p) {
    const ushort4x r = *(const ushort4x*)p;
    return make_float4(bf16_to_f32(r.v[0]), bf16_to_f32(r.v[1]),
                       bf16_to_f32(r.v[2]), bf16_to_f32(r.v[3]));
  }
  static DEVINLINE void st(uint16_t* p, float4 v) {
    ushort4x r;
    r.v[0] = f32_to_bf16(v.x);
    r.v[1] = f32_to_bf16(v.y);
    r.v[2] = f32_to_bf16(v.z);
    r.v[3] = f32_to_bf16(v.w);
    *(ushort4x*)p = r;
  }
};

DEVINLINE float4 axpy4(float a, float4 x, float4 y) {
  return make_float4(a * x.x + y.x, a * x.y + y.y, a * x.z + y.z,
                     a * x.w + y.w);
}

// One block per row; a thread owns NV groups of four neighbouring columns
// in every stream, so a row's old streams, its new ones and the normed
// input all live in registers between one read and one write of memory.
template <typename TD, typename TO, int B, int NV>
__global__ __launch_bounds__(ST_BLOCK) void stream_step_kernel(
    TO* __restrict__ out, const float* src, int64_t src_rs, int64_t src_ss,
    float* dst, const TD* __restrict__ y, int64_t y_rs,
    const float* __restrict__ mix, const float* __restrict__ outw,
    const float* __restrict__ inw, const float* __restrict__ norm_w, int D,
    float eps) {
  __shared__ float red[8];
  const int64_t t = blockIdx.x;
  const float* xs = src + t * src_rs;
  float4 u[NV], x[B], nx[B];
  float ss = 0.0f;
  auto fetch = [&](int v, float4* to) {
    const int d = (v * ST_BLOCK + threadIdx.x) * 4;
#pragma unroll
    for (int b = 0; b < B; ++b)
      to[b] = d < D ? *(const float4*)(xs + b * src_ss + d)
                    : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  };
  fetch(0, nx);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * ST_BLOCK + threadIdx.x) * 4;
#pragma unroll
    for (int b = 0; b < B; ++b) x[b] = nx[b];
    // the next columns are requested before these are stored (dst may be
    // src, so the compiler keeps the order written here)
    if (v + 1 < NV) fetch(v + 1, nx);
    float4 acc = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (d < D) {
      if (y != nullptr) {
        const float4 yy = Act4<TD>::ld(y + t * y_rs + d);
#pragma unroll
        for (int e = 0; e < B; ++e) {
          const float c = outw[e];
          float4 n = make_float4(c * yy.x, c * yy.y, c * yy.z, c * yy.w);
#pragma unroll
          for (int b = 0; b < B; ++b) n = axpy4(mix[b * B + e], x[b], n);
          *(float4*)(dst + (t * B + e) * D + d) = n;
          acc = axpy4(inw[e], n, acc);
        }
      } else {
#pragma unroll
        for (int b = 0; b < B; ++b) acc = axpy4(inw[b], x[b], acc);
      }
      ss += acc.x * acc.x + acc.y * acc.y + acc.z * acc.z + acc.w * acc.w;
    }
    u[v] = acc;
  }
  ss = block_reduce_sum<ST_BLOCK>(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)D + eps);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int d = (v * ST_BLOCK + threadIdx.x) * 4;
    if (d >= D) continue;
    const float4 w = *(const float4*)(norm_w + d);
    Act4<TO>::st(out + t * D + d,
                 make_float4(u[v].x * r * w.x, u[v].y * r * w.y,
                             u[v].z * r * w.z, u[v].w * r * w.w));
  }
}

// any number of streams, any width; dst is never src
template <typename TD, typename TO>
__global__ __launch_bounds__(ST_BLOCK) void stream_step_any_kernel(
    TO* __restrict__ out, const float* __restrict__ src, int64_t src_rs,
    int64_t src_ss, float* __restrict__ dst, const TD* __restrict__ y,
    int64_t y_rs, const float* __restrict__ mix,
    const float* __restrict__ outw, const float* __restrict__ inw,
    const float* __restrict__ norm_w, int B, int D, float eps) {
  __shared__ float red[8];
  const int64_t t = blockIdx.x;
  const float* xs = src + t * src_rs;
  float ss = 0.0f;
  for (int d = threadIdx.x; d < D; d += ST_BLOCK) {
    float acc = 0.0f;
    if (y != nullptr) {
      const float yy = Act<TD>::ld(y + t * y_rs + d);
      for (int e = 0; e < B; ++e) {
        float n = outw[e] * yy;
        for (int b = 0; b < B; ++b) n += mix[b * B + e] * xs[b * src_ss + d];
        dst[(t * B + e) * D + d] = n;
        acc += inw[e] * n;
      }
    } else {
      for (int b = 0; b < B; ++b) acc += inw[b] * xs[b * src_ss + d];
    }
    ss += acc * acc;
  }
  ss = block_reduce_sum<ST_BLOCK>(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)D + eps);
  // a thread reads back only what it wrote
  for (int d = threadIdx.x; d < D; d += ST_BLOCK) {
    float acc = 0.0f;
    for (int b = 0; b < B; ++b)
      acc += inw[b] * (y != nullptr ? dst[(t * B + b) * D + d]
                                    : xs[b * src_ss + d]);
    Act<TO>::st(out + t * D + d, acc * r * norm_w[d]);
  }
}

// widest stream count of the register kernel; more streams need dst != src
int64_t stream_step_max_in_place() { return 8; }

void stream_step(torch::Tensor out, torch::Tensor src,
                 c10::optional<torch::Tensor> dst,
                 c10::optional<torch::Tensor> y,
                 c10::optional<torch::Tensor> mix,
                 c10::optional<torch::Tensor> outw, torch::Tensor inw,
                 torch::Tensor norm_w, double eps) {
  TORCH_CHECK(src.is_cuda() && src.dtype() == torch::kFloat32 &&
              src.dim() == 3 && src.stride(2) == 1);
  const int T = src.size(0), B = src.size(1), D = src.size(2);
  TORCH_CHECK(out.is_contiguous() && out.dim() == 2 && out.size(0) == T &&
              out.size(1) == D);
  auto fvec = [&](const torch::Tensor& t, int64_t n) {
    TORCH_CHECK(t.is_cuda() && t.dtype() == torch::kFloat32 &&
                t.is_contiguous() && t.numel() == n);
  };
  fvec(inw, B);
  fvec(norm_w, D);
  bool y16 = false;
  bool in_place = false;
  if (y.has_value()) {
    TORCH_CHECK(dst.has_value() && mix.has_value() && outw.has_value());
    fvec(*mix, (int64_t)B * B);
    fvec(*outw, B);
    TORCH_CHECK(dst->dtype() == torch::kFloat32 && dst->is_contiguous() &&
                dst->sizes() == src.sizes());
    TORCH_CHECK(y->dim() == 2 && y->size(0) == T && y->size(1) == D &&
                y->stride(1) == 1);
    y16 = y->scalar_type() == torch::kBFloat16;
    TORCH_CHECK(y16 || y->scalar_type() == torch::kFloat32,
                "the sublayer's result must be bfloat16 or float32");
    in_place = dst->data_ptr() == src.data_ptr();
    TORCH_CHECK(!in_place || src.is_contiguous(),
                "repeated streams are not updated in place");
  }
  if (T == 0) return;
  hipStream_t stream = at::cuda::getCurrentCUDAStream();
  const int64_t ye = y.has_value() ? y->element_size() : 2;
  auto al = [](const void* p, int64_t n) {
    return reinterpret_cast<uintptr_t>(p) % n == 0;
  };
  const bool regs =
      B <= stream_step_max_in_place() && D % 4 == 0 &&
      D <= 8 * 4 * ST_BLOCK && src.stride(0) % 4 == 0 &&
      src.stride(1) % 4 == 0 && al(src.data_ptr(), 16) &&
      al(norm_w.data_ptr(), 16) && al(out.data_ptr(), 16) &&
      (!y.has_value() || (y->stride(0) % 4 == 0 &&
                          al(y->data_ptr(), 4 * ye) &&
                          al(dst->data_ptr(), 16)));
  TORCH_CHECK(regs || !in_place,
              "this stream count or width is not updated in place");
  const int nv = (D + 4 * ST_BLOCK - 1) / (4 * ST_BLOCK);
#define ST_ARGS(TD, TO)                                                       \
  (TO*)out.data_ptr(), (const float*)src.data_ptr(), (int64_t)src.stride(0),  \
      (int64_t)src.stride(1),                                                 \
      y.has_value() ? (float*)dst->data_ptr() : nullptr,                      \
      y.has_value() ? (const TD*)y->data_ptr() : nullptr,                     \
      y.has_value() ? (int64_t)y->stride(0) : 0,                              \
      y.has_value() ? (const float*)mix->data_ptr() : nullptr,                \
      y.has_value() ? (const float*)outw->data_ptr() : nullptr,               \
      (const float*)inw.data_ptr(), (const float*)norm_w.data_ptr()
#define ST_LAUNCH(TD, TO, BV, NVV)                                            \
  hipLaunchKernelGGL((stream_step_kernel<TD, TO, BV, NVV>), dim3(T),          \
                     dim3(ST_BLOCK), 0, stream, ST_ARGS(TD, TO), D,           \
                     (float)eps)
#define ST_NV(TD, TO, BV)                                                     \
  do {                                                                        \
    if (nv <= 1) ST_LAUNCH(TD, TO, BV, 1);                                    \
    else if (nv <= 2) ST_LAUNCH(TD, TO, BV, 2);                               \
    else if (nv <= 4) ST_LAUNCH(TD, TO, BV, 4);                               \
    else ST_LAUNCH(TD, TO, BV, 8);                                            \
  } while (0)
#define ST_B(TD, TO)                                                          \
  do {                                                                        \
    if (!regs) {                                                              \
      hipLaunchKernelGGL((stream_step_any_kernel<TD, TO>), dim3(T),           \
                         dim3(ST_BLOCK), 0, stream, ST_ARGS(TD, TO), B, D,    \
                         (float)eps);                                         \
      break;                                                                  \
    }                                                                         \
    switch (B) {                                                              \
      case 1: ST_NV(TD, TO, 1); break;                                        \
      case 2: ST_NV(TD, TO, 2); break;                                        \
      case 3: ST_NV(TD, TO, 3); break;                                        \
      case 4: ST_NV(TD, TO, 4); break;                                        \
      case 5: ST_NV(TD, TO, 5); break;                                        \
      case 6: ST_NV(TD, TO, 6); break;                                        \
      case 7: ST_NV(TD, TO, 7); break;                                        \
      default: ST_NV(TD, TO, 8); break;                                       \
    }                                                                         \
  } while (0)
  IGW_DISPATCH_ACT(out, {
    if (y.has_value())
      TORCH_CHECK(y->scalar_type() == out.scalar_type(),
                  "the sublayer's result and the output share a type");
    ST_B(act_t, act_t);
  });
#undef ST_B
#undef ST_NV
#undef ST_LAUNCH
#undef ST_ARGS
  HIP_CHECK_KERNEL();
}

// ---------------------------------------------------------------------------
// expert dispatch: one block per (token, choice) row, 16-byte pieces where
// the layout allows
template <typename T, bool V4>
__global__ __launch_bounds__(256) void moe_scatter_rows_kernel(
    T* __restrict__ buf, const T* __restrict__ x, int64_t x_rs,
    const int64_t* __restrict__ dst, int K, int D) {
  const int64_t a = blockIdx.x;
  const T* s = x + (a / K) * x_rs;
  T* o = buf + dst[a] * D;
  if constexpr (V4) {
    for (int d = threadIdx.x * 4; d < D; d += 1024)
      Act4<T>::st(o + d, Act4<T>::ld(s + d));
  } else {
    for (int d = threadIdx.x; d < D; d += 256) o[d] = s[d];
  }
}

void moe_scatter_rows(torch::Tensor buf, torch::Tensor x, torch::Tensor dst,
                      int64_t K) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.stride(1) == 1);
  const int64_t T = x.size(0);
  const int D = x.size(1);
  TORCH_CHECK(buf.is_contiguous() && buf.dim() == 2 && buf.size(1) == D &&
              buf.dtype() == x.dtype());
  TORCH_CHECK(K >= 1 && dst.dtype() == torch::kInt64 &&
              dst.is_contiguous() && dst.numel() == T * K);
  if (T == 0) return;
  hipStream_t stream = at::cuda::getCurrentCUDAStream();
  const bool v4 = D % 4 == 0 && x.stride(0) % 4 == 0 &&
                  reinterpret_cast<uintptr_t>(x.data_ptr()) % 16 == 0;
#define MSC(V)                                                                \
  hipLaunchKernelGGL((moe_scatter_rows_kernel<act_t, V>),                     \
                     dim3((unsigned)(T * K)), dim3(256), 0, stream,           \
                     (act_t*)buf.data_ptr(), (const act_t*)x.data_ptr(),      \
                     (int64_t)x.stride(0), (const int64_t*)dst.data_ptr(),    \
                     (int)K, D)
  IGW_DISPATCH_ACT(x, {
    if (v4) MSC(true);
    else MSC(false);
  });
#undef MSC
  HIP_CHECK_KERNEL();
}

// one block per token
template <typename T, bool V4>
__global__ __launch_bounds__(256) void moe_combine_kernel(
    T* __restrict__ out, const T* __restrict__ y,
    const int64_t* __restrict__ dst, const float* __restrict__ w,
    const T* __restrict__ shared, const float* __restrict__ g, int64_t g_rs,
    int K, int D) {
  const int64_t t = blockIdx.x;
  const int64_t* rows = dst + t * K;
  const float* wt = w + t * K;
  const float sg = shared != nullptr ? sigmoid_f32(g[t * g_rs]) : 0.0f;
  if constexpr (V4) {
    for (int d = threadIdx.x * 4; d < D; d += 1024) {
      float4 acc = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
      for (int k = 0; k < K; ++k)
        acc = axpy4(wt[k], Act4<T>::ld(y + rows[k] * D + d), acc);
      if (shared != nullptr)
        acc = axpy4(sg, Act4<T>::ld(shared + t * D + d), acc);
      Act4<T>::st(out + t * D + d, acc);
    }
  } else {
    for (int d = threadIdx.x; d < D; d += 256) {
      float acc = 0.0f;
      for (int k = 0; k < K; ++k)
        acc += wt[k] * Act<T>::ld(y + rows[k] * D + d);
      if (shared != nullptr) acc += sg * Act<T>::ld(shared + t * D + d);
      Act<T>::st(out + t * D + d, acc);
    }
  }
}

void moe_combine(torch::Tensor out, torch::Tensor y, torch::Tensor dst,
                 torch::Tensor w, c10::optional<torch::Tensor> shared,
                 c10::optional<torch::Tensor> g) {
  TORCH_CHECK(y.is_cuda() && y.dim() == 2 && y.is_contiguous());
  const int D = y.size(1);
  TORCH_CHECK(w.dtype() == torch::kFloat32 && w.is_contiguous() &&
              w.dim() == 2);
  const int64_t T = w.size(0);
  const int K = w.size(1);
  TORCH_CHECK(dst.dtype() == torch::kInt64 && dst.is_contiguous() &&
              dst.numel() == T * K);
  TORCH_CHECK(out.is_contiguous() && out.dtype() == y.dtype() &&
              out.dim() == 2 && out.size(0) == T && out.size(1) == D);
  TORCH_CHECK(shared.has_value() == g.has_value());
  if (shared.has_value()) {
    TORCH_CHECK(shared->is_contiguous() && shared->dtype() == y.dtype() &&
                shared->sizes() == out.sizes());
    TORCH_CHECK(g->dtype() == torch::kFloat32 && g->dim() == 1 &&
                g->size(0) == T);
  }
  if (T == 0) return;
  hipStream_t stream = at::cuda::getCurrentCUDAStream();
#define MCB(V)                                                                \
  hipLaunchKernelGGL(                                                         \
      (moe_combine_kernel<act_t, V>), dim3((unsigned)T), dim3(256), 0,        \
      stream, (act_t*)out.data_ptr(), (const act_t*)y.data_ptr(),             \
      (const int64_t*)dst.data_ptr(), (const float*)w.data_ptr(),             \
      shared.has_value() ? (const act_t*)shared->data_ptr() : nullptr,        \
      g.has_value() ? (const float*)g->data_ptr() : nullptr,                  \
      g.has_value() ? (int64_t)g->stride(0) : 0, K, D)
  IGW_DISPATCH_ACT(y, {
    if (D % 4 == 0) MCB(true);
    else MCB(false);
  });
#undef MCB
  HIP_CHECK_KERNEL();
}

}  // namespace igw
