// The boundary between two sublayers of a decoder whose residual stream is fp32 and whose sublayers
// are normalised on both sides (a norm on the sublayer's output before it joins the residual, a
// norm on the residual before the next sublayer):
//   x <- x + branch_scale * post_gain * y * rsqrt(mean(y^2) + eps)
//   h  = next_scale * next_gain * x * rsqrt(mean(x^2) + eps), or next_scale * x without a gain
// in one launch: y is read once, x is read and written once, h leaves in the activations' type. The
// first sublayer's input takes the same kernel without a post norm (x = scale * embedding row).
// Where the sublayer is a mixture of experts, y is summed up on the fly from the chosen experts'
// outputs and their weights (mui_moe_residual_norm), so that no combined tensor is ever written.
#include "common.cuh"

namespace mui {

constexpr int kRnThreads = 256;

struct ResidualNormParams {
  const float* residual_in;  // [rows, k] or null (0)
  const void* y;             // [rows, k] (dense sublayer output), activations' type
  float y_scale;
  const void* post_gain;  // [k] or null: y joins the residual as y_scale * y
  float branch_scale;     // on the normed y
  const void* next_gain;  // [k] or null: h is the sum itself
  float next_scale;
  float eps;
  float* residual_out;  // [rows, k], may be residual_in
  void* h;              // [rows, k] or null
  int k;
  // mixture of experts: y[r] = sum_j weight[r, j] * (expert[r, j] < n_experts ? pairs[r * top + j] : identity[r])
  const void* pairs;
  const void* identity;
  const int* expert;
  const float* weight;
  int n_experts, top;
};

__device__ __forceinline__ float rn_block_sum(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();  // the previous use of red is over
  if ((threadIdx.x & (kWave - 1)) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}

// k % 8 == 0, 16-byte aligned rows, k <= 8 * 256 * CH: the row stays in registers
template <typename T, int CH, bool MOE>
__global__ void __launch_bounds__(kRnThreads) residual_norm_vec_kernel(const ResidualNormParams p) {
  typedef typename T::storage S;
  __shared__ float red[kRnThreads / kWave];
  const int t = threadIdx.x;
  const long row = blockIdx.x, base = row * p.k;
  const int kc = p.k >> 3;
  float x[CH][8], y[CH][8];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < CH; ++j) {
    const int c = t + kRnThreads * j;
    if (c < kc) {
#pragma unroll
      for (int i = 0; i < 8; ++i) x[j][i] = 0.f;
      if (p.residual_in) load8<F32>(p.residual_in + base + (c << 3), x[j]);
      if constexpr (!MOE) {
        load8<T>((const S*)p.y + base + (c << 3), y[j]);
#pragma unroll
        for (int i = 0; i < 8; ++i) y[j][i] *= p.y_scale;
      } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) y[j][i] = 0.f;
      }
    }
  }
  if constexpr (MOE) {
    // four experts' rows requested together
    for (int s0 = 0; s0 < p.top; s0 += 4) {
      const S* src[4];
      float w[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int s = s0 + u < p.top ? s0 + u : p.top - 1;
        const int e = p.expert[row * p.top + s];
        w[u] = s0 + u < p.top ? p.weight[row * p.top + s] : 0.f;
        src[u] = e < p.n_experts ? (const S*)p.pairs + (row * p.top + s) * p.k : (const S*)p.identity + base;
      }
#pragma unroll
      for (int j = 0; j < CH; ++j) {
        const int c = t + kRnThreads * j;
        if (c < kc) {
          float f[4][8];
#pragma unroll
          for (int u = 0; u < 4; ++u) load8<T>(src[u] + (c << 3), f[u]);
#pragma unroll
          for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int i = 0; i < 8; ++i) y[j][i] = fmaf(w[u], f[u][i], y[j][i]);
        }
      }
    }
  }
  if (p.post_gain) {
#pragma unroll
    for (int j = 0; j < CH; ++j)
      if (t + kRnThreads * j < kc)
#pragma unroll
        for (int i = 0; i < 8; ++i) ss = fmaf(y[j][i], y[j][i], ss);
    const float rs = rsqrtf(rn_block_sum(ss, red) / (float)p.k + p.eps);
#pragma unroll
    for (int j = 0; j < CH; ++j) {
      const int c = t + kRnThreads * j;
      if (c < kc) {
        float g[8];
        load8<T>((const S*)p.post_gain + (c << 3), g);
#pragma unroll
        for (int i = 0; i < 8; ++i) x[j][i] = fmaf(g[i] * p.branch_scale, y[j][i] * rs, x[j][i]);
      }
    }
  } else {
#pragma unroll
    for (int j = 0; j < CH; ++j)
#pragma unroll
      for (int i = 0; i < 8; ++i) x[j][i] += y[j][i];
  }
  ss = 0.f;
#pragma unroll
  for (int j = 0; j < CH; ++j) {
    const int c = t + kRnThreads * j;
    if (c < kc) {
      store8<F32>(p.residual_out + base + (c << 3), x[j]);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss = fmaf(x[j][i], x[j][i], ss);
    }
  }
  if (!p.h) return;
  const float rs = p.next_gain ? rsqrtf(rn_block_sum(ss, red) / (float)p.k + p.eps) * p.next_scale : p.next_scale;
#pragma unroll
  for (int j = 0; j < CH; ++j) {
    const int c = t + kRnThreads * j;
    if (c < kc) {
      float g[8], o[8];
      if (p.next_gain) {
        load8<T>((const S*)p.next_gain + (c << 3), g);
      } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) g[i] = 1.f;
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) o[i] = g[i] * (x[j][i] * rs);
      store8<T>((S*)p.h + base + (c << 3), o);
    }
  }
}

// any k, any alignment; every thread comes back to the elements it handled before
template <typename T, bool MOE>
__global__ void __launch_bounds__(kRnThreads) residual_norm_any_kernel(const ResidualNormParams p) {
  typedef typename T::storage S;
  __shared__ float red[kRnThreads / kWave];
  const int t = threadIdx.x;
  const long row = blockIdx.x, base = row * p.k;
  auto y_at = [&](int i) -> float {
    if constexpr (MOE) {
      float y = 0.f;
      for (int s = 0; s < p.top; ++s) {
        const int e = p.expert[row * p.top + s];
        const float v = e < p.n_experts ? T::one(((const S*)p.pairs)[(row * p.top + s) * p.k + i])
                                        : T::one(((const S*)p.identity)[base + i]);
        y = fmaf(p.weight[row * p.top + s], v, y);
      }
      return y;
    } else {
      return p.y_scale * T::one(((const S*)p.y)[base + i]);
    }
  };
  float rs = 1.f;
  if (p.post_gain) {
    float ss = 0.f;
    for (int i = t; i < p.k; i += kRnThreads) {
      const float y = y_at(i);
      ss = fmaf(y, y, ss);
    }
    rs = rsqrtf(rn_block_sum(ss, red) / (float)p.k + p.eps);
  }
  float ss = 0.f;
  for (int i = t; i < p.k; i += kRnThreads) {
    float x = p.residual_in ? p.residual_in[base + i] : 0.f;
    const float y = y_at(i);
    x = p.post_gain ? fmaf(T::one(((const S*)p.post_gain)[i]) * p.branch_scale, y * rs, x) : x + y;
    p.residual_out[base + i] = x;
    ss = fmaf(x, x, ss);
  }
  if (!p.h) return;
  rs = p.next_gain ? rsqrtf(rn_block_sum(ss, red) / (float)p.k + p.eps) * p.next_scale : p.next_scale;
  for (int i = t; i < p.k; i += kRnThreads)
    ((S*)p.h)[base + i] = T::pack((p.next_gain ? T::one(((const S*)p.next_gain)[i]) : 1.f) * (p.residual_out[base + i] * rs));
}

template <typename T, bool MOE>
static int launch_residual_norm(hipStream_t s, const ResidualNormParams& p, int rows) {
  const void* ptrs[] = {p.residual_in, p.y, p.post_gain, p.next_gain, p.residual_out, p.h, p.pairs, p.identity};
  bool vec = p.k % 8 == 0 && p.k <= 8 * 8 * kRnThreads;
  for (const void* q : ptrs) vec = vec && aligned16(q);
  const dim3 grid(rows), block(kRnThreads);
  if (!vec) {
    hipLaunchKernelGGL((residual_norm_any_kernel<T, MOE>), grid, block, 0, s, p);
  } else {
    const int ch = ceil_div(p.k >> 3, kRnThreads);
    if (ch <= 1) hipLaunchKernelGGL((residual_norm_vec_kernel<T, 1, MOE>), grid, block, 0, s, p);
    else if (ch <= 2) hipLaunchKernelGGL((residual_norm_vec_kernel<T, 2, MOE>), grid, block, 0, s, p);
    else if (ch <= 4) hipLaunchKernelGGL((residual_norm_vec_kernel<T, 4, MOE>), grid, block, 0, s, p);
    else hipLaunchKernelGGL((residual_norm_vec_kernel<T, 8, MOE>), grid, block, 0, s, p);
  }
  return launch_status();
}

template <bool MOE>
static int dispatch_residual_norm(mui_stream_t stream, int dtype, const ResidualNormParams& p, int rows) {
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MUI_DTYPE_F16) return launch_residual_norm<F16, MOE>(s, p, rows);
  if (dtype == MUI_DTYPE_BF16) return launch_residual_norm<BF16, MOE>(s, p, rows);
  if (dtype == MUI_DTYPE_F32) return launch_residual_norm<F32, MOE>(s, p, rows);
  return MUI_ERR_INVALID_ARG;
}

}  // namespace mui

using namespace mui;

extern "C" int mui_residual_norm(mui_stream_t stream, int dtype, const float* residual_in, const void* y, float y_scale,
                                 const void* post_gain, float branch_scale, const void* next_gain, float next_scale,
                                 float epsilon, float* residual_out, void* h, int rows, int k) {
  MUI_CHECK_ARG(y && residual_out && rows > 0 && k > 0 && (h || !next_gain));
  ResidualNormParams p = {};
  p.residual_in = residual_in; p.y = y; p.y_scale = y_scale; p.post_gain = post_gain; p.next_gain = next_gain;
  p.branch_scale = branch_scale; p.next_scale = next_scale; p.eps = epsilon; p.residual_out = residual_out; p.h = h; p.k = k;
  return dispatch_residual_norm<false>(stream, dtype, p, rows);
}

extern "C" int mui_moe_residual_norm(mui_stream_t stream, int dtype, const float* residual_in, const void* pair_out,
                                     const void* identity_in, const int32_t* expert, const float* weight, int n_experts,
                                     int top, const void* post_gain, float branch_scale, const void* next_gain,
                                     float next_scale, float epsilon, float* residual_out, void* h, int rows, int k) {
  MUI_CHECK_ARG(pair_out && identity_in && expert && weight && residual_out && rows > 0 && k > 0);
  MUI_CHECK_ARG(n_experts >= 0 && top > 0 && (h || !next_gain));
  ResidualNormParams p = {};
  p.residual_in = residual_in; p.y_scale = 1.f; p.post_gain = post_gain; p.next_gain = next_gain;
  p.branch_scale = branch_scale; p.next_scale = next_scale; p.eps = epsilon; p.residual_out = residual_out; p.h = h; p.k = k;
  p.pairs = pair_out; p.identity = identity_in; p.expert = expert; p.weight = weight; p.n_experts = n_experts; p.top = top;
  return dispatch_residual_norm<true>(stream, dtype, p, rows);
}
