// Shared device helpers of the sequence-mixing kernels (gfx950, wave64).
// Kernels are templated on the matrix dtype T (bf16 or float); everything
// that carries state, a norm, a score or the residual is float.
#pragma once

#include <hip/hip_runtime.h>
#include <hip/hip_bf16.h>
#include <cstdint>

#define SM_WAVE 64
#define SM_INLINE __device__ __forceinline__

typedef __hip_bfloat16 bf16_t;

SM_INLINE float to_f(float x) { return x; }
SM_INLINE float to_f(bf16_t x) { return __bfloat162float(x); }
template <typename T> SM_INLINE T from_f(float x);
template <> SM_INLINE float from_f<float>(float x) { return x; }
template <> SM_INLINE bf16_t from_f<bf16_t>(float x) { return __float2bfloat16(x); }

SM_INLINE float sm_wave_sum(float x) {
  #pragma unroll
  for (int off = 32; off > 0; off >>= 1) x += __shfl_xor(x, off, SM_WAVE);
  return x;
}
SM_INLINE float sm_wave_max(float x) {
  #pragma unroll
  for (int off = 32; off > 0; off >>= 1) x = fmaxf(x, __shfl_xor(x, off, SM_WAVE));
  return x;
}
// Reductions over the 16 lanes of a row (lanes that share lane >> 4) on the
// VALU's lane-permute path: the two quad swaps, then the mirrors of 8 and of
// 16 lanes; afterwards every lane of the row holds the result.
template <int CTRL> SM_INLINE float sm_dpp(float x) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), CTRL, 0xf, 0xf, true));
}
SM_INLINE float sm_row16_max(float x) {
  x = fmaxf(x, sm_dpp<0xB1>(x));    // quad_perm [1, 0, 3, 2]
  x = fmaxf(x, sm_dpp<0x4E>(x));    // quad_perm [2, 3, 0, 1]
  x = fmaxf(x, sm_dpp<0x141>(x));   // row_half_mirror
  return fmaxf(x, sm_dpp<0x140>(x));   // row_mirror
}
SM_INLINE float sm_row16_sum(float x) {
  x += sm_dpp<0xB1>(x);
  x += sm_dpp<0x4E>(x);
  x += sm_dpp<0x141>(x);
  return x + sm_dpp<0x140>(x);
}
// Sum over a block of up to 1024 threads; red needs blockDim.x / 64 floats.
SM_INLINE float sm_block_sum(float x, float* red) {
  const int lane = threadIdx.x & (SM_WAVE - 1), wid = threadIdx.x / SM_WAVE;
  const int nw = (blockDim.x + SM_WAVE - 1) / SM_WAVE;
  x = sm_wave_sum(x);
  __syncthreads();
  if (lane == 0) red[wid] = x;
  __syncthreads();
  float r = 0.f;
  for (int i = 0; i < nw; ++i) r += red[i];
  return r;
}
SM_INLINE float sm_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
// The same on the hardware's exponential and reciprocal: relative error of about
// (2 + |z|) 2^-24.
SM_INLINE float sm_fast_sigmoid(float z) {
  return __builtin_amdgcn_rcpf(1.0f + __expf(-z));
}
// 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))), fp32 inside.
SM_INLINE float gelu_tanh_f(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
// VEC (1 or 4) neighbouring row entries as fp32, one access each.
template <int VEC> struct sm_vec { float v[VEC]; };

template <int VEC> SM_INLINE sm_vec<VEC> sm_load(const float* p) {
  sm_vec<VEC> r;
  if constexpr (VEC == 4) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    r.v[0] = a.x; r.v[1] = a.y; r.v[2] = a.z; r.v[3] = a.w;
  } else {
    r.v[0] = *p;
  }
  return r;
}
template <int VEC> SM_INLINE sm_vec<VEC> sm_load(const bf16_t* p) {
  sm_vec<VEC> r;
  if constexpr (VEC == 4) {
    const uint2 a = *reinterpret_cast<const uint2*>(p);
    r.v[0] = __uint_as_float(a.x << 16); r.v[1] = __uint_as_float(a.x & 0xffff0000u);
    r.v[2] = __uint_as_float(a.y << 16); r.v[3] = __uint_as_float(a.y & 0xffff0000u);
  } else {
    r.v[0] = to_f(*p);
  }
  return r;
}
template <int VEC> SM_INLINE void sm_store(float* p, const sm_vec<VEC>& r) {
  if constexpr (VEC == 4) *reinterpret_cast<float4*>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
  else *p = r.v[0];
}
template <int VEC> SM_INLINE void sm_store(bf16_t* p, const sm_vec<VEC>& r) {
  if constexpr (VEC == 4) {
    unsigned int w[4];
    #pragma unroll
    for (int k = 0; k < 4; ++k) w[k] = __bfloat16_as_ushort(__float2bfloat16(r.v[k]));
    *reinterpret_cast<uint2*>(p) = make_uint2(w[0] | (w[1] << 16), w[2] | (w[3] << 16));
  } else {
    *p = __float2bfloat16(r.v[0]);
  }
}
// Differential attention: lam_w = lq1 | lk1 | lq2 | lk2 (dk entries each);
// lambda = exp(lq1.lk1) - exp(lq2.lk2) + diff, the difference's norm takes eps.
struct wa_diff {
  const float* lam_w;
  float diff, eps;
};
// Every lane of the wave takes part and gets lambda.
SM_INLINE float wa_lambda(const wa_diff& df, int dk, int lane) {
  float s1 = 0.f, s2 = 0.f;
  for (int k = lane; k < dk; k += SM_WAVE) {
    s1 = fmaf(df.lam_w[k], df.lam_w[dk + k], s1);
    s2 = fmaf(df.lam_w[2 * dk + k], df.lam_w[3 * dk + k], s2);
  }
  return expf(sm_wave_sum(s1)) - expf(sm_wave_sum(s2)) + df.diff;
}
// Which keys a query sees besides j <= p: the last `window` positions (0: all),
// its own chunk of `chunk` positions (0: no chunks) and the first `keep` tokens;
// how its scores close: cap tanh(score / cap) (0: as they are) and a per-head
// sink that joins the softmax denominator (null: none).
struct wa_view {
  int window, chunk, keep;
  float cap;
  const float* sink;
};
// First position of the range that ends at p.
SM_INLINE int wa_first(const wa_view& v, int p) {
  int lo = (v.window > 0 && p - v.window + 1 > 0) ? p - v.window + 1 : 0;
  if (v.chunk > 0) lo = max(lo, p / v.chunk * v.chunk);
  return lo;
}
// What the sink adds to a softmax sum taken relative to the maximum m.
SM_INLINE float wa_sink(const wa_view& v, int head, float m) {
  return v.sink != nullptr ? expf(v.sink[head] - m) : 0.f;
}
// clamped GLU: g = min(gate, limit), u = clamp(up, +-limit), g sigmoid(1.702 g) (u + 1)
SM_INLINE float sm_capped_glu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sm_sigmoid(1.702f * g) * (u + 1.0f);
}

#define SM_CHECK_LAUNCH()                                                  \
  do {                                                                     \
    hipError_t e_ = hipGetLastError();                                     \
    TORCH_CHECK(e_ == hipSuccess, "HIP kernel launch failed: ",            \
                hipGetErrorString(e_));                                    \
  } while (0)

#define SM_CDIV(a, b) (((a) + (b) - 1) / (b))

#define SM_CHECK_CUDA(t) TORCH_CHECK((t).is_cuda() && (t).is_contiguous(), #t " must be a contiguous GPU tensor")
#define SM_CHECK_F32(t) TORCH_CHECK((t).scalar_type() == at::kFloat, #t " must be float32")
#define SM_CHECK_I32(t) TORCH_CHECK((t).scalar_type() == at::kInt, #t " must be int32")
