// Residual streams (hyper-connections). A token's residual is S fp32 rows
// x_1 .. x_S of width D, stored [token][stream][D]. A sublayer reads
// norm(sum_s read[s] x_s); its output s enters every stream:
//   x_t <- sum_s mix[s, t] x_s + out[t] s        (all from the old streams)
//   hyper_start      embedding row * scale into every stream, first norm
//   hyper_residual   closes a sublayer and opens the next: optional RMS norm
//                    of each of two addends (the sides of a parallel pair),
//                    their scaled sum, the stream update in place, the next
//                    read sum and its norm; the streams are read and written
//                    once
//   hyper_close      norm(sum_s x_s) of selected rows
// The norm is an RMS norm, or (center) a layer norm: mean taken off, variance
// from the deviations (the read sum waits in LDS, so the second pass costs no
// memory traffic). One workgroup per token row; VEC entries per access.
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>
#include "seqmix_common.h"

namespace {

// h = norm(u) * w for the row u in LDS; every thread handles the entries it
// wrote itself (same stride), sum is its share of the row's sum.
template <typename T, int VEC>
SM_INLINE void hs_norm_out(const float* u, float sum, const float* __restrict__ w, float eps,
                           bool center, int D, float* red, T* __restrict__ h) {
  const float mean = center ? sm_block_sum(sum, red) / (float)D : 0.f;
  float ss = 0.f;
  for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
    const sm_vec<VEC> v = sm_load<VEC>(u + d);
    #pragma unroll
    for (int k = 0; k < VEC; ++k) ss += (v.v[k] - mean) * (v.v[k] - mean);
  }
  const float inv = 1.0f / sqrtf(sm_block_sum(ss, red) / (float)D + eps);
  for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
    sm_vec<VEC> v = sm_load<VEC>(u + d);
    const sm_vec<VEC> wv = sm_load<VEC>(w + d);
    #pragma unroll
    for (int k = 0; k < VEC; ++k) v.v[k] = (v.v[k] - mean) * inv * wv.v[k];
    sm_store<VEC>(h + d, v);
  }
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void hyper_start_kernel(
    const T* __restrict__ embed, const int64_t* __restrict__ tokens, float scale, int S,
    const float* __restrict__ read_w, const float* __restrict__ norm_w, float eps, int center,
    int D, float* __restrict__ x, T* __restrict__ h) {
  extern __shared__ __attribute__((aligned(16))) float hs_u[];
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const T* e = embed + tokens[t] * D;
  float sum = 0.f;
  for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
    sm_vec<VEC> v = sm_load<VEC>(e + d), u;
    #pragma unroll
    for (int k = 0; k < VEC; ++k) { v.v[k] *= scale; u.v[k] = 0.f; }
    for (int s = 0; s < S; ++s) {
      sm_store<VEC>(x + (t * S + s) * D + d, v);
      const float r = read_w[s];
      #pragma unroll
      for (int k = 0; k < VEC; ++k) u.v[k] = fmaf(r, v.v[k], u.v[k]);
    }
    #pragma unroll
    for (int k = 0; k < VEC; ++k) sum += u.v[k];
    sm_store<VEC>(hs_u + d, u);
  }
  hs_norm_out<T, VEC>(hs_u, sum, norm_w, eps, center != 0, D, red, h + t * D);
}

// SMAX: streams held in registers; exact for up to 4, above that the loops
// are guarded by the actual count.
template <typename T, typename TY, int SMAX, int VEC>
__global__ __launch_bounds__(256) void hyper_residual_kernel(
    float* __restrict__ x, const TY* __restrict__ y, const TY* __restrict__ y2,
    const float* __restrict__ yw, const float* __restrict__ y2w, float ys, float y2s,
    const float* __restrict__ mix, const float* __restrict__ out_w,
    const float* __restrict__ read_w, const float* __restrict__ norm_w, float eps, int center,
    int S_, int D, T* __restrict__ h) {
  extern __shared__ __attribute__((aligned(16))) float hs_u[];
  __shared__ float red[4];
  const int S = (SMAX <= 4) ? SMAX : S_;
  const int64_t t = blockIdx.x;
  const TY* yr = y + t * D;
  const TY* y2r = (y2 != nullptr) ? y2 + t * D : nullptr;
  float a = ys, a2 = y2s;
  if (yw != nullptr || y2w != nullptr) {
    float ss = 0.f, ss2 = 0.f;
    for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
      const sm_vec<VEC> v = sm_load<VEC>(yr + d);
      #pragma unroll
      for (int k = 0; k < VEC; ++k) ss += v.v[k] * v.v[k];
      if (y2r != nullptr) {
        const sm_vec<VEC> v2 = sm_load<VEC>(y2r + d);
        #pragma unroll
        for (int k = 0; k < VEC; ++k) ss2 += v2.v[k] * v2.v[k];
      }
    }
    if (yw != nullptr) a *= 1.0f / sqrtf(sm_block_sum(ss, red) / (float)D + eps);
    if (y2w != nullptr) a2 *= 1.0f / sqrtf(sm_block_sum(ss2, red) / (float)D + eps);
  }
  float* xr = x + t * S * D;
  float sum = 0.f;
  for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
    sm_vec<VEC> xs[SMAX];
    #pragma unroll
    for (int s = 0; s < SMAX; ++s)
      if (s < S) xs[s] = sm_load<VEC>(xr + (int64_t)s * D + d);
    sm_vec<VEC> v = sm_load<VEC>(yr + d);
    if (yw != nullptr) {
      const sm_vec<VEC> w = sm_load<VEC>(yw + d);
      #pragma unroll
      for (int k = 0; k < VEC; ++k) v.v[k] *= w.v[k];
    }
    #pragma unroll
    for (int k = 0; k < VEC; ++k) v.v[k] *= a;
    if (y2r != nullptr) {
      sm_vec<VEC> v2 = sm_load<VEC>(y2r + d);
      if (y2w != nullptr) {
        const sm_vec<VEC> w = sm_load<VEC>(y2w + d);
        #pragma unroll
        for (int k = 0; k < VEC; ++k) v2.v[k] *= w.v[k];
      }
      #pragma unroll
      for (int k = 0; k < VEC; ++k) v.v[k] = fmaf(a2, v2.v[k], v.v[k]);
    }
    sm_vec<VEC> u;
    #pragma unroll
    for (int k = 0; k < VEC; ++k) u.v[k] = 0.f;
    #pragma unroll
    for (int q = 0; q < SMAX; ++q) {
      if (q < S) {
        sm_vec<VEC> n;
        const float o = out_w[q];
        #pragma unroll
        for (int k = 0; k < VEC; ++k) n.v[k] = o * v.v[k];
        #pragma unroll
        for (int s = 0; s < SMAX; ++s) {
          if (s < S) {
            const float m = mix[s * S + q];
            #pragma unroll
            for (int k = 0; k < VEC; ++k) n.v[k] = fmaf(m, xs[s].v[k], n.v[k]);
          }
        }
        sm_store<VEC>(xr + (int64_t)q * D + d, n);
        if (norm_w != nullptr) {
          const float r = read_w[q];
          #pragma unroll
          for (int k = 0; k < VEC; ++k) u.v[k] = fmaf(r, n.v[k], u.v[k]);
        }
      }
    }
    if (norm_w != nullptr) {
      #pragma unroll
      for (int k = 0; k < VEC; ++k) sum += u.v[k];
      sm_store<VEC>(hs_u + d, u);
    }
  }
  if (norm_w != nullptr)
    hs_norm_out<T, VEC>(hs_u, sum, norm_w, eps, center != 0, D, red, h + t * D);
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void hyper_close_kernel(
    const float* __restrict__ x, const int64_t* __restrict__ rows, int64_t T_rows, int S,
    const float* __restrict__ norm_w, float eps, int center, int D, T* __restrict__ h) {
  extern __shared__ __attribute__((aligned(16))) float hs_u[];
  __shared__ float red[4];
  const int64_t row = rows[blockIdx.x];
  if (row < 0 || row >= T_rows) return;            // uniform over the workgroup
  float sum = 0.f;
  for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
    sm_vec<VEC> u = sm_load<VEC>(x + row * S * D + d);
    for (int s = 1; s < S; ++s) {
      const sm_vec<VEC> v = sm_load<VEC>(x + (row * S + s) * D + d);
      #pragma unroll
      for (int k = 0; k < VEC; ++k) u.v[k] += v.v[k];
    }
    #pragma unroll
    for (int k = 0; k < VEC; ++k) sum += u.v[k];
    sm_store<VEC>(hs_u + d, u);
  }
  hs_norm_out<T, VEC>(hs_u, sum, norm_w, eps, center != 0, D, red,
                      h + (int64_t)blockIdx.x * D);
}

const float* f32_ptr(const torch::Tensor& t, int64_t n, const char* what) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == at::kFloat && t.numel() == n,
              "hyper streams: ", what, " must be a contiguous float32 GPU tensor of ", n, " entries");
  return t.data_ptr<float>();
}

void check_width(int64_t D) {
  TORCH_CHECK(D >= 1 && D <= 16384, "hyper streams: width above 16384");
}

}  // namespace

#define HS_MAX_STREAMS 16

std::vector<torch::Tensor> hyper_start(torch::Tensor embed, torch::Tensor tokens, double scale,
                                       int64_t streams, torch::Tensor read_w, torch::Tensor norm_w,
                                       double eps, bool out_bf16, bool center) {
  SM_CHECK_CUDA(embed); SM_CHECK_CUDA(tokens);
  TORCH_CHECK(embed.dim() == 2 && tokens.dim() == 1 && tokens.scalar_type() == at::kLong,
              "hyper_start: embed [V, D], int64 tokens");
  const bool bf16 = embed.scalar_type() == at::kBFloat16;
  if (!bf16) SM_CHECK_F32(embed);
  TORCH_CHECK(bf16 == out_bf16, "hyper_start: the output dtype is the embedding's");
  TORCH_CHECK(streams >= 1 && streams <= HS_MAX_STREAMS, "hyper_start: streams");
  const int64_t T = tokens.numel();
  const int D = embed.size(1), S = streams;
  check_width(D);
  const float* rp = f32_ptr(read_w, S, "read weights");
  const float* np = f32_ptr(norm_w, D, "norm weight");
  auto x = torch::empty({T, S, D}, embed.options().dtype(at::kFloat));
  auto h = torch::empty({T, D}, embed.options());
  if (T == 0) return {x, h};
  auto stream = at::cuda::getCurrentCUDAStream();
#define HS_START(TY, VEC)                                                                      \
  hyper_start_kernel<TY, VEC><<<T, 256, D * sizeof(float), stream>>>(                          \
      reinterpret_cast<const TY*>(embed.data_ptr()), tokens.data_ptr<int64_t>(), (float)scale, \
      S, rp, np, (float)eps, center ? 1 : 0, D, x.data_ptr<float>(),                           \
      reinterpret_cast<TY*>(h.data_ptr()))
  if (bf16) { if (D % 4 == 0) HS_START(bf16_t, 4); else HS_START(bf16_t, 1); }
  else { if (D % 4 == 0) HS_START(float, 4); else HS_START(float, 1); }
#undef HS_START
  SM_CHECK_LAUNCH();
  return {x, h};
}

c10::optional<torch::Tensor> hyper_residual_norm(
    torch::Tensor x, torch::Tensor y, c10::optional<torch::Tensor> y2,
    c10::optional<torch::Tensor> y_w, c10::optional<torch::Tensor> y2_w, double y_scale,
    double y2_scale, torch::Tensor mix, torch::Tensor out_w, c10::optional<torch::Tensor> read_w,
    c10::optional<torch::Tensor> norm_w, double eps, bool out_bf16, bool center) {
  SM_CHECK_CUDA(x); SM_CHECK_F32(x); SM_CHECK_CUDA(y);
  TORCH_CHECK(x.dim() == 3, "hyper_residual_norm: x is [T, S, D]");
  const int64_t T = x.size(0);
  const int S = x.size(1), D = x.size(2);
  TORCH_CHECK(S >= 1 && S <= HS_MAX_STREAMS, "hyper_residual_norm: streams");
  check_width(D);
  TORCH_CHECK(y.dim() == 2 && y.size(0) == T && y.size(1) == D, "hyper_residual_norm: y shape");
  const bool yb = y.scalar_type() == at::kBFloat16;
  if (!yb) SM_CHECK_F32(y);
  const void* y2p = nullptr;
  torch::Tensor y2c;
  if (y2.has_value()) {
    y2c = y2->to(y.scalar_type());
    SM_CHECK_CUDA(y2c);
    TORCH_CHECK(y2c.dim() == 2 && y2c.size(0) == T && y2c.size(1) == D, "hyper_residual_norm: y2 shape");
    y2p = y2c.data_ptr();
  }
  const float* yw = y_w.has_value() ? f32_ptr(*y_w, D, "y norm weight") : nullptr;
  const float* y2w = (y2_w.has_value() && y2p != nullptr) ? f32_ptr(*y2_w, D, "y2 norm weight") : nullptr;
  const float* mp = f32_ptr(mix, (int64_t)S * S, "mix");
  const float* op = f32_ptr(out_w, S, "output weights");
  const float* rp = nullptr;
  const float* np = nullptr;
  c10::optional<torch::Tensor> h;
  if (norm_w.has_value()) {
    TORCH_CHECK(read_w.has_value(), "hyper_residual_norm: the next read needs its stream weights");
    rp = f32_ptr(*read_w, S, "read weights");
    np = f32_ptr(*norm_w, D, "norm weight");
    h = torch::empty({T, D}, x.options().dtype(out_bf16 ? at::kBFloat16 : at::kFloat));
  }
  if (T == 0) return h;
  auto stream = at::cuda::getCurrentCUDAStream();
  void* hp = h.has_value() ? h->data_ptr() : nullptr;
  const size_t lds = np != nullptr ? D * sizeof(float) : 0;
#define HS_RES(TO, TY, N, VEC)                                                               \
  hyper_residual_kernel<TO, TY, N, VEC><<<T, 256, lds, stream>>>(                            \
      x.data_ptr<float>(), reinterpret_cast<const TY*>(y.data_ptr()),                        \
      reinterpret_cast<const TY*>(y2p), yw, y2w, (float)y_scale, (float)y2_scale, mp, op,    \
      rp, np, (float)eps, center ? 1 : 0, S, D, reinterpret_cast<TO*>(hp))
#define HS_RES_S(TO, TY, VEC)                      \
  do {                                             \
    if (S == 1) HS_RES(TO, TY, 1, VEC);            \
    else if (S == 2) HS_RES(TO, TY, 2, VEC);       \
    else if (S == 3) HS_RES(TO, TY, 3, VEC);       \
    else if (S == 4) HS_RES(TO, TY, 4, VEC);       \
    else if (S <= 8) HS_RES(TO, TY, 8, VEC);       \
    else HS_RES(TO, TY, 16, VEC);                  \
  } while (0)
#define HS_RES_V(TO, TY)                           \
  do {                                             \
    if (D % 4 == 0) HS_RES_S(TO, TY, 4);           \
    else HS_RES_S(TO, TY, 1);                      \
  } while (0)
  if (out_bf16) { if (yb) HS_RES_V(bf16_t, bf16_t); else HS_RES_V(bf16_t, float); }
  else {
    TORCH_CHECK(!yb, "hyper_residual_norm: fp32 output needs fp32 addends");
    HS_RES_V(float, float);
  }
#undef HS_RES_V
#undef HS_RES_S
#undef HS_RES
  SM_CHECK_LAUNCH();
  return h;
}

torch::Tensor hyper_close_norm(torch::Tensor x, torch::Tensor rows, torch::Tensor norm_w, double eps,
                               bool out_bf16, bool center) {
  SM_CHECK_CUDA(x); SM_CHECK_F32(x); SM_CHECK_CUDA(rows);
  TORCH_CHECK(x.dim() == 3 && rows.dim() == 1 && rows.scalar_type() == at::kLong,
              "hyper_close_norm: x [T, S, D], int64 rows");
  const int64_t n = rows.numel();
  const int S = x.size(1), D = x.size(2);
  check_width(D);
  const float* np = f32_ptr(norm_w, D, "norm weight");
  auto h = torch::empty({n, (int64_t)D}, x.options().dtype(out_bf16 ? at::kBFloat16 : at::kFloat));
  if (n == 0) return h;
  auto stream = at::cuda::getCurrentCUDAStream();
#define HS_CLOSE(TY, VEC)                                                                     \
  hyper_close_kernel<TY, VEC><<<n, 256, D * sizeof(float), stream>>>(                         \
      x.data_ptr<float>(), rows.data_ptr<int64_t>(), x.size(0), S, np, (float)eps,            \
      center ? 1 : 0, D, reinterpret_cast<TY*>(h.data_ptr()))
  if (out_bf16) { if (D % 4 == 0) HS_CLOSE(bf16_t, 4); else HS_CLOSE(bf16_t, 1); }
  else { if (D % 4 == 0) HS_CLOSE(float, 4); else HS_CLOSE(float, 1); }
#undef HS_CLOSE
  SM_CHECK_LAUNCH();
  return h;
}
