// Between the input projection and the absorbed query of a latent
// attention layer whose queries come straight from the layer input
// (gfx950), one launch:
//
//   x [T, H*(dn+rd) | R | rd]      the fused projection's row
//   c = x[R part] / sqrt(mean(.^2) + eps) * w   -> cache row [0, R)
//   shared key part, rotated                    -> cache row [R, R + rd)
//   the last rd entries of every query head are rotated in place
//
// pairs (2i, 2i+1), or HALF (i, i + n_pairs), turn by position * inv_freq;
// cos and sin (times mag) are evaluated once per row into LDS and serve
// the key and all heads.  One 256-thread block per row, fp32 arithmetic.
#include "../csrc_hybrid/act_types.h"

namespace igw {

template <typename T>
__global__ __launch_bounds__(256) void latent_rope_append_kernel(
    T* __restrict__ x, int64_t x_rs, const int32_t* __restrict__ positions,
    const int32_t* __restrict__ slot_mapping, T* __restrict__ cache,
    const float* __restrict__ w, const float* __restrict__ inv_freq,
    int n_pairs, int half, float mag, float eps, int H, int dn, int rd,
    int R) {
  extern __shared__ float cs[];
  __shared__ float red[8];
  const int64_t t = blockIdx.x;
  T* row = x + t * x_rs;
  const T* c = row + (int64_t)H * (dn + rd);
  const T* kr = c + R;
  const float pos = (float)positions[t];
  for (int i = threadIdx.x; i < n_pairs; i += 256) {
    const float ang = pos * inv_freq[i];
    cs[i] = cosf(ang) * mag;
    cs[n_pairs + i] = sinf(ang) * mag;
  }
  float ss = 0.0f;
  for (int d = threadIdx.x; d < R; d += 256) {
    const float v = Act<T>::ld(c + d);
    ss += v * v;
  }
  // its barriers also publish cs
  ss = block_reduce_sum<256>(ss, red);
  const float r = 1.0f / sqrtf(ss / (float)R + eps);
  T* crow = cache + (int64_t)slot_mapping[t] * (R + rd);
  for (int d = threadIdx.x; d < R; d += 256)
    Act<T>::st(crow + d, Act<T>::ld(c + d) * r * w[d]);
  for (int d = 2 * n_pairs + threadIdx.x; d < rd; d += 256)
    crow[R + d] = kr[d];
  // unit 0 is the shared key, units 1 .. H the query heads
  for (int i = threadIdx.x; i < n_pairs * (H + 1); i += 256) {
    const int u = i / n_pairs, p = i - u * n_pairs;
    const int a = half ? p : 2 * p, b = half ? p + n_pairs : 2 * p + 1;
    T* q = row + (int64_t)(u - 1) * (dn + rd) + dn;
    const T* s = u == 0 ? kr : q;
    T* o = u == 0 ? crow + R : q;
    const float va = Act<T>::ld(s + a), vb = Act<T>::ld(s + b);
    const float co = cs[p], si = cs[n_pairs + p];
    Act<T>::st(o + a, va * co - vb * si);
    Act<T>::st(o + b, vb * co + va * si);
  }
}

void latent_rope_append(torch::Tensor x, torch::Tensor positions,
                        torch::Tensor slot_mapping, torch::Tensor cache,
                        torch::Tensor norm_w, torch::Tensor inv_freq,
                        double eps, int64_t heads, int64_t dim,
                        int64_t rot_dim, int64_t kv_rank, bool half,
                        double mag) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && x.stride(1) == 1);
  const int T = x.size(0);
  TORCH_CHECK(x.size(1) == heads * (dim + rot_dim) + kv_rank + rot_dim);
  TORCH_CHECK(cache.is_contiguous() && cache.dim() == 3 &&
              cache.size(2) == kv_rank + rot_dim &&
              cache.dtype() == x.dtype());
  TORCH_CHECK(positions.dtype() == torch::kInt32 && positions.numel() == T &&
              slot_mapping.dtype() == torch::kInt32 &&
              slot_mapping.numel() == T);
  TORCH_CHECK(norm_w.dtype() == torch::kFloat32 && norm_w.is_contiguous() &&
              norm_w.numel() == kv_rank);
  const int n_pairs = inv_freq.numel();
  TORCH_CHECK(inv_freq.dtype() == torch::kFloat32 &&
              inv_freq.is_contiguous() && 2 * n_pairs <= rot_dim &&
              n_pairs <= 4096);
  if (T == 0) return;
  hipStream_t stream = at::cuda::getCurrentCUDAStream();
  IGW_DISPATCH_ACT(x, {
    hipLaunchKernelGGL((latent_rope_append_kernel<act_t>), dim3(T), dim3(256),
                       (size_t)(2 * n_pairs) * sizeof(float), stream,
                       (act_t*)x.data_ptr(), (int64_t)x.stride(0),
                       (const int32_t*)positions.data_ptr(),
                       (const int32_t*)slot_mapping.data_ptr(),
                       (act_t*)cache.data_ptr(),
                       (const float*)norm_w.data_ptr(),
                       (const float*)inv_freq.data_ptr(), n_pairs,
                       half ? 1 : 0, (float)mag, (float)eps, (int)heads,
                       (int)dim, (int)rot_dim, (int)kv_rank);
  });
  HIP_CHECK_KERNEL();
}

}  // namespace igw
