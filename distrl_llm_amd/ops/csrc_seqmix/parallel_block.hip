// Parallel block: one norm feeds mixer and feed-forward, x += mixer + ff.
//   parallel_start     embedding row * scale (+ a vector) -> fp32 residual, first
//                      norm
//   parallel_residual  layer tail: optional RMS norm of each of two mixer addends
//                      (the sides of a parallel pair), their scaled sum and the
//                      feed-forward into the residual; what a pass of a loop adds
//                      at its start (the embedding row again, read from the table,
//                      and a learned vector); the next layer's norm
// The norms that the next layer reads carry the weight as (offset + w). One
// workgroup per token row; the residual is read and written once and waits in
// LDS for the second pass of the norm.
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>
#include "seqmix_common.h"

namespace {

// h = u / rms(u) * (offset + w) for the row u in LDS; every thread reads the
// entries it wrote itself, ss is its share of the row's sum of squares.
template <typename T, int VEC>
SM_INLINE void pb_norm_out(const float* u, float ss, const float* __restrict__ w, float eps,
                           float offset, int D, float* red, T* __restrict__ h) {
  const float inv = 1.0f / sqrtf(sm_block_sum(ss, red) / (float)D + eps);
  for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
    sm_vec<VEC> v = sm_load<VEC>(u + d);
    const sm_vec<VEC> wv = sm_load<VEC>(w + d);
    #pragma unroll
    for (int k = 0; k < VEC; ++k) v.v[k] = v.v[k] * inv * (offset + wv.v[k]);
    sm_store<VEC>(h + d, v);
  }
}

// What is added at the start of a pass. embed null: the vector only.
template <typename T> struct pb_inject {
  const T* embed;             // [V, D]
  const int64_t* tokens;      // [Tn]
  int64_t V;
  float scale;
  const float* step;          // [D]
};

template <typename T>
SM_INLINE const T* pb_row(const pb_inject<T>& in, int64_t t, int D) {
  if (in.embed == nullptr) return nullptr;
  int64_t id = in.tokens[t];
  id = id < 0 ? 0 : (id >= in.V ? in.V - 1 : id);    // ids stay inside the table
  return in.embed + id * D;
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void parallel_start_kernel(
    pb_inject<T> in, const float* __restrict__ norm_w, float eps, float offset, int D,
    float* __restrict__ x, T* __restrict__ h) {
  extern __shared__ __attribute__((aligned(16))) float pb_u[];
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const T* e = pb_row(in, t, D);
  float ss = 0.f;
  for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
    sm_vec<VEC> v = sm_load<VEC>(e + d);
    #pragma unroll
    for (int k = 0; k < VEC; ++k) v.v[k] *= in.scale;
    if (in.step != nullptr) {
      const sm_vec<VEC> s = sm_load<VEC>(in.step + d);
      #pragma unroll
      for (int k = 0; k < VEC; ++k) v.v[k] += s.v[k];
    }
    #pragma unroll
    for (int k = 0; k < VEC; ++k) ss += v.v[k] * v.v[k];
    sm_store<VEC>(x + t * D + d, v);
    sm_store<VEC>(pb_u + d, v);
  }
  pb_norm_out<T, VEC>(pb_u, ss, norm_w, eps, offset, D, red, h + t * D);
}

template <typename T, typename TF, int VEC>
__global__ __launch_bounds__(256) void parallel_residual_kernel(
    float* __restrict__ x, const T* __restrict__ y, const T* __restrict__ y2,
    const float* __restrict__ yw, const float* __restrict__ y2w, float ys, float y2s,
    const TF* __restrict__ f, pb_inject<T> in, const float* __restrict__ norm_w, float eps,
    float offset, int D, T* __restrict__ h) {
  extern __shared__ __attribute__((aligned(16))) float pb_u[];
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const T* yr = (y != nullptr) ? y + t * D : nullptr;
  const T* y2r = (y2 != nullptr) ? y2 + t * D : nullptr;
  const TF* fr = (f != nullptr) ? f + t * D : nullptr;
  const T* er = pb_row(in, t, D);
  float a = ys, a2 = y2s;
  if (yw != nullptr || y2w != nullptr) {
    float ss = 0.f, ss2 = 0.f;
    for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
      if (yw != nullptr) {
        const sm_vec<VEC> v = sm_load<VEC>(yr + d);
        #pragma unroll
        for (int k = 0; k < VEC; ++k) ss += v.v[k] * v.v[k];
      }
      if (y2w != nullptr) {
        const sm_vec<VEC> v = sm_load<VEC>(y2r + d);
        #pragma unroll
        for (int k = 0; k < VEC; ++k) ss2 += v.v[k] * v.v[k];
      }
    }
    if (yw != nullptr) a *= 1.0f / sqrtf(sm_block_sum(ss, red) / (float)D + eps);
    if (y2w != nullptr) a2 *= 1.0f / sqrtf(sm_block_sum(ss2, red) / (float)D + eps);
  }
  float xx = 0.f;
  for (int d = threadIdx.x * VEC; d < D; d += blockDim.x * VEC) {
    sm_vec<VEC> v = sm_load<VEC>(x + t * D + d);
    auto add = [&](sm_vec<VEC> s, const float* w, float f1) {
      if (w != nullptr) {
        const sm_vec<VEC> wv = sm_load<VEC>(w + d);
        #pragma unroll
        for (int k = 0; k < VEC; ++k) s.v[k] *= wv.v[k];
      }
      #pragma unroll
      for (int k = 0; k < VEC; ++k) v.v[k] = fmaf(f1, s.v[k], v.v[k]);
    };
    if (yr != nullptr) add(sm_load<VEC>(yr + d), yw, a);
    if (y2r != nullptr) add(sm_load<VEC>(y2r + d), y2w, a2);
    if (fr != nullptr) add(sm_load<VEC>(fr + d), nullptr, 1.0f);
    if (er != nullptr) add(sm_load<VEC>(er + d), nullptr, in.scale);
    if (in.step != nullptr) add(sm_load<VEC>(in.step + d), nullptr, 1.0f);
    sm_store<VEC>(x + t * D + d, v);
    if (norm_w != nullptr) {
      #pragma unroll
      for (int k = 0; k < VEC; ++k) xx += v.v[k] * v.v[k];
      sm_store<VEC>(pb_u + d, v);
    }
  }
  if (norm_w != nullptr)
    pb_norm_out<T, VEC>(pb_u, xx, norm_w, eps, offset, D, red, h + t * D);
}

const float* row_f32(const c10::optional<torch::Tensor>& t, int64_t n, const char* what) {
  if (!t.has_value()) return nullptr;
  TORCH_CHECK(t->is_cuda() && t->is_contiguous() && t->scalar_type() == at::kFloat && t->numel() == n,
              "parallel block: ", what, " must be a contiguous float32 GPU tensor of ", n, " entries");
  return t->data_ptr<float>();
}

void check_width(int64_t D) {
  TORCH_CHECK(D >= 1 && D <= 16384, "parallel block: width above 16384");
}

}  // namespace

std::vector<torch::Tensor> parallel_start(torch::Tensor embed, torch::Tensor tokens, double scale,
                                          c10::optional<torch::Tensor> step, torch::Tensor norm_w,
                                          double eps, bool out_bf16, double offset) {
  SM_CHECK_CUDA(embed); SM_CHECK_CUDA(tokens);
  TORCH_CHECK(embed.dim() == 2 && embed.size(0) >= 1 && tokens.dim() == 1 &&
              tokens.scalar_type() == at::kLong, "parallel_start: embed [V, D], int64 tokens");
  const bool bf16 = embed.scalar_type() == at::kBFloat16;
  if (!bf16) SM_CHECK_F32(embed);
  TORCH_CHECK(bf16 == out_bf16, "parallel_start: the output dtype is the embedding's");
  const int64_t T = tokens.numel();
  const int D = embed.size(1);
  check_width(D);
  const float* sp = row_f32(step, D, "step");
  const float* np = row_f32(norm_w, D, "norm weight");
  auto x = torch::empty({T, D}, embed.options().dtype(at::kFloat));
  auto h = torch::empty({T, D}, embed.options());
  if (T == 0) return {x, h};
  auto stream = at::cuda::getCurrentCUDAStream();
#define PB_START(TY, VEC)                                                                     \
  parallel_start_kernel<TY, VEC><<<T, 256, D * sizeof(float), stream>>>(                      \
      pb_inject<TY>{reinterpret_cast<const TY*>(embed.data_ptr()), tokens.data_ptr<int64_t>(), \
                    embed.size(0), (float)scale, sp},                                         \
      np, (float)eps, (float)offset, D, x.data_ptr<float>(), reinterpret_cast<TY*>(h.data_ptr()))
  if (bf16) { if (D % 4 == 0) PB_START(bf16_t, 4); else PB_START(bf16_t, 1); }
  else { if (D % 4 == 0) PB_START(float, 4); else PB_START(float, 1); }
#undef PB_START
  SM_CHECK_LAUNCH();
  return {x, h};
}

c10::optional<torch::Tensor> parallel_residual_norm(
    torch::Tensor x, c10::optional<torch::Tensor> y, c10::optional<torch::Tensor> y2,
    c10::optional<torch::Tensor> y_w, c10::optional<torch::Tensor> y2_w, double y_scale,
    double y2_scale, c10::optional<torch::Tensor> f, c10::optional<torch::Tensor> embed,
    c10::optional<torch::Tensor> tokens, double scale, c10::optional<torch::Tensor> step,
    c10::optional<torch::Tensor> norm_w, double eps, bool out_bf16, double offset) {
  SM_CHECK_CUDA(x); SM_CHECK_F32(x);
  TORCH_CHECK(x.dim() == 2, "parallel_residual_norm: x is [T, D]");
  const int64_t T = x.size(0);
  const int D = x.size(1);
  check_width(D);
  const auto mdt = out_bf16 ? at::kBFloat16 : at::kFloat;
  auto rows = [&](const c10::optional<torch::Tensor>& t, const char* what) -> const void* {
    if (!t.has_value()) return nullptr;
    TORCH_CHECK(t->is_cuda() && t->is_contiguous() && t->dim() == 2 && t->size(0) == T &&
                t->size(1) == D, "parallel_residual_norm: ", what, " must be a contiguous [T, D]");
    return t->data_ptr();
  };
  const void* yp = rows(y, "y");
  const void* y2p = rows(y2, "y2");
  const void* fp = rows(f, "f");
  TORCH_CHECK((yp == nullptr || y->scalar_type() == mdt) && (y2p == nullptr || y2->scalar_type() == mdt),
              "parallel_residual_norm: the mixer's outputs are in the model dtype");
  const bool fb = fp != nullptr && f->scalar_type() == at::kBFloat16;
  if (fp != nullptr && !fb) SM_CHECK_F32(*f);
  TORCH_CHECK(!fb || out_bf16, "parallel_residual_norm: bf16 feed-forward in a fp32 model");
  const float* yw = yp != nullptr ? row_f32(y_w, D, "y norm weight") : nullptr;
  const float* y2w = y2p != nullptr ? row_f32(y2_w, D, "y2 norm weight") : nullptr;
  const float* sp = row_f32(step, D, "step");
  const void* ep = nullptr;
  const int64_t* tp = nullptr;
  int64_t V = 0;
  if (embed.has_value()) {
    TORCH_CHECK(tokens.has_value(), "parallel_residual_norm: the embedding needs its tokens");
    SM_CHECK_CUDA(*embed); SM_CHECK_CUDA(*tokens);
    TORCH_CHECK(embed->dim() == 2 && embed->size(0) >= 1 && embed->size(1) == D &&
                embed->scalar_type() == mdt && tokens->numel() == T &&
                tokens->scalar_type() == at::kLong, "parallel_residual_norm: embedding");
    ep = embed->data_ptr();
    tp = tokens->data_ptr<int64_t>();
    V = embed->size(0);
  }
  const float* np = row_f32(norm_w, D, "norm weight");
  c10::optional<torch::Tensor> h;
  if (np != nullptr) h = torch::empty({T, D}, x.options().dtype(mdt));
  if (T == 0) return h;
  auto stream = at::cuda::getCurrentCUDAStream();
  void* hp = h.has_value() ? h->data_ptr() : nullptr;
  const size_t lds = np != nullptr ? D * sizeof(float) : 0;
#define PB_RES(TY, TF, VEC)                                                                   \
  parallel_residual_kernel<TY, TF, VEC><<<T, 256, lds, stream>>>(                             \
      x.data_ptr<float>(), reinterpret_cast<const TY*>(yp), reinterpret_cast<const TY*>(y2p), \
      yw, y2w, (float)y_scale, (float)y2_scale, reinterpret_cast<const TF*>(fp),              \
      pb_inject<TY>{reinterpret_cast<const TY*>(ep), tp, V, (float)scale, sp}, np, (float)eps, \
      (float)offset, D, reinterpret_cast<TY*>(hp))
#define PB_RES_V(TY, TF) do { if (D % 4 == 0) PB_RES(TY, TF, 4); else PB_RES(TY, TF, 1); } while (0)
  if (!out_bf16) PB_RES_V(float, float);
  else if (fb) PB_RES_V(bf16_t, bf16_t);
  else PB_RES_V(bf16_t, float);
#undef PB_RES_V
#undef PB_RES
  SM_CHECK_LAUNCH();
  return h;
}
