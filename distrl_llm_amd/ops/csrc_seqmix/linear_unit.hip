// Real-gated linear recurrent unit over a flat varlen batch, fp32 vector state
// per slot. Projection rows [y | x] (W channels each, biases added):
//   u = conv(x) + bias (short, causal, depthwise; inputs before the portion come
//       from tails[slot])
//   r, i = sigmoid of block-diagonal maps of u (n x n matrices)
//   log a = -c r softplus(lam),  S <- a S + sqrt(1 - a^2) i u
//   out = S gelu_tanh(y)
// Kernels:
//   linear_unit_tile   bf16 prompt steps, one workgroup per (tile of <= 64
//                      tokens of a sequence, block, 64 or 128 channels): convolution
//                      into LDS, both gates on MFMA (u as two bf16 terms, hi +
//                      lo), then the recurrence inside the tile as prefixes
//                      (P_t, Q_t): S_t = P_t S_start + Q_t
//   linear_unit_carry  S_start of a row's tiles in order, new state
//   linear_unit_apply  S_t and the output branch
//   linear_unit_step   bf16 steps of one token per row: convolution, gates on
//                      MFMA, state and output in one kernel
//   linear_unit_plain, linear_unit_walk   fp32 models and odd sizes
// The tails are advanced afterwards (every kernel above only reads them).
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>
#include "seqmix_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16v8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

namespace {

struct lu_args {
  int64_t ldp;                    // projection row pitch
  int W, n, taps;                 // channels, channels per block
  const float *conv_w, *conv_b;   // [W, taps], [W]
  const float* tails;             // [slots, taps - 1, W]
  const float* gates_b;           // [2, W]
  const float* lam;               // [W]
  float c;
  const int *cu, *tok_seq, *slots;
};

SM_INLINE float lu_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// Decay a and input b = sqrt(1 - a^2) i u from the gates' pre-activations.
SM_INLINE void lu_gate(const lu_args& A, int ch, float zr, float zi, float u, float* a, float* b) {
  const float r = sm_sigmoid(zr + A.gates_b[ch]), i = sm_sigmoid(zi + A.gates_b[A.W + ch]);
  const float la = -A.c * r * lu_softplus(A.lam[ch]);
  *a = expf(la);
  *b = sqrtf(-expm1f(2.0f * la)) * i * u;
}

// The same for the bf16 kernels on the hardware's exponential, reciprocal and
// square root, with what depends on the channel only (biases, c softplus(lam))
// taken once: errors of a few fp32 roundings. 1 - a^2 = -expm1(2 log a) by its
// series where the exponential would cancel.
struct lu_channel { float br, bi, csp; };
SM_INLINE lu_channel lu_channel_of(const lu_args& A, int ch) {
  return {A.gates_b[ch], A.gates_b[A.W + ch], A.c * lu_softplus(A.lam[ch])};
}
SM_INLINE void lu_gate_fast(const lu_channel& C, float zr, float zi, float u, float* a, float* b) {
  const float la = -C.csp * sm_fast_sigmoid(zr + C.br);
  const float e = 2.0f * la;
  float p = fmaf(e, 1.0f / 7.0f, 1.0f);
  p = fmaf(e * (1.0f / 6.0f), p, 1.0f);
  p = fmaf(e * (1.0f / 5.0f), p, 1.0f);
  p = fmaf(e * (1.0f / 4.0f), p, 1.0f);
  p = fmaf(e * (1.0f / 3.0f), p, 1.0f);
  p = fmaf(e * (1.0f / 2.0f), p, 1.0f);
  const float x = __expf(la);
  const float left = (e > -0.25f) ? -e * p : fmaf(-x, x, 1.0f);
  *a = x;
  *b = __builtin_amdgcn_sqrtf(left) * sm_fast_sigmoid(zi + C.bi) * u;
}

// u of channel ch for the token whose x row starts at xr, rel tokens into its
// portion; tl: the slot's tails.
template <typename T>
SM_INLINE float lu_conv(const lu_args& A, const T* xr, int rel, const float* tl, int ch) {
  const float* w = A.conv_w + (int64_t)ch * A.taps;
  float acc = A.conv_b[ch];
  for (int j = 0; j < A.taps; ++j) {
    const int back = A.taps - 1 - j;
    const float v = (rel >= back) ? to_f(xr[ch - (int64_t)back * A.ldp])
                                  : tl[(int64_t)(j + rel) * A.W + ch];
    acc = fmaf(w[j], v, acc);
  }
  return acc;
}
// Eight neighbouring channels ch .. ch + 7 (16-byte pieces). TAPS > 0: that
// many taps, unrolled.
template <int TAPS>
SM_INLINE void lu_conv8(const lu_args& A, const bf16_t* xr, int rel, const float* tl, int ch,
                        const float* wr, float* u) {
  const int taps = TAPS > 0 ? TAPS : A.taps;
  #pragma unroll
  for (int e = 0; e < 8; ++e) u[e] = A.conv_b[ch + e];
  #pragma unroll
  for (int j = 0; j < taps; ++j) {
    const int back = taps - 1 - j;
    float v[8];
    if (rel >= back) {
      const bf16v8 p = *reinterpret_cast<const bf16v8*>(xr + ch - (int64_t)back * A.ldp);
      #pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = (float)p[e];
    } else {
      const float* q = tl + (int64_t)(j + rel) * A.W + ch;
      #pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = q[e];
    }
    #pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float w = TAPS > 0 ? wr[e * taps + j] : A.conv_w[(int64_t)(ch + e) * taps + j];
      u[e] = fmaf(w, v[e], u[e]);
    }
  }
}
SM_INLINE void lu_split(const float* u, bf16v8* hi, bf16v8* lo) {
  #pragma unroll
  for (int e = 0; e < 8; ++e) {
    (*hi)[e] = (__bf16)u[e];
    (*lo)[e] = (__bf16)(u[e] - (float)(*hi)[e]);
  }
}

// ---- prompt tiles
#define LUT_KC 128            // channels of a block staged at once
#define LUT_KP (LUT_KC + 8)
// NW waves, 16 channels each: with 8 the block's convolution is redone half as
// often.
template <int TAPS, int NW>
__global__ __launch_bounds__(64 * NW, 2) void linear_unit_tile_kernel(
    const bf16_t* __restrict__ x,         // x part of the projection rows
    const bf16_t* __restrict__ gw,        // [2, blocks, n, n]
    const int* __restrict__ tiles,        // [ntiles, 3] = (row, first token, tokens)
    lu_args A, float* __restrict__ P, float* __restrict__ Q) {
  __shared__ __attribute__((aligned(16))) __bf16 uh[64 * LUT_KP];
  __shared__ __attribute__((aligned(16))) __bf16 ul[64 * LUT_KP];
  constexpr int NC = 16 * NW;
  __shared__ float own[64][NC + 1];       // fp32 u of the workgroup's own channels
  const int b = tiles[3 * blockIdx.x], t0 = tiles[3 * blockIdx.x + 1], nt = tiles[3 * blockIdx.x + 2];
  const int blk = blockIdx.y, c0 = blockIdx.z * NC, n = A.n;
  const int tid = threadIdx.x, wave = tid >> 6, l = tid & 63, lrow = l & 15, lk = l >> 4;
  const int rel0 = t0 - A.cu[b];
  const float* tl = A.tails + (int64_t)A.slots[b] * (A.taps - 1) * A.W;
  const int col = c0 + wave * 16 + lrow;             // the lane's channel in the block
  const bf16_t* w0 = gw + ((int64_t)blk * n + min(col, n - 1)) * n;
  const bf16_t* w1 = w0 + (int64_t)A.W * n;
  f32x4 acc[2][4];
  #pragma unroll
  for (int g = 0; g < 2; ++g)
    #pragma unroll
    for (int mt = 0; mt < 4; ++mt) acc[g][mt] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < n; k0 += LUT_KC) {
    __syncthreads();
    // convolution: a thread takes 8 channels for a few neighbouring tokens
    {
      const int kc = (tid & 15) * 8, ch = blk * n + k0 + kc;
      const bool in = k0 + kc < n;
      float wr[TAPS > 0 ? 8 * TAPS : 1];
      if (TAPS > 0 && in) {
        #pragma unroll
        for (int e = 0; e < 8 * TAPS; ++e) wr[e] = A.conv_w[(int64_t)ch * TAPS + e];
      }
      #pragma unroll
      for (int s = 0; s < 16 / NW; ++s) {
        const int tok = (tid >> 4) * (16 / NW) + s;
        float u[8];
        #pragma unroll
        for (int e = 0; e < 8; ++e) u[e] = 0.f;
        if (in && tok < nt)
          lu_conv8<TAPS>(A, x + (int64_t)(t0 + tok) * A.ldp, rel0 + tok, tl, ch, wr, u);
        bf16v8 hi, lo;
        lu_split(u, &hi, &lo);
        *reinterpret_cast<bf16v8*>(uh + tok * LUT_KP + kc) = hi;
        *reinterpret_cast<bf16v8*>(ul + tok * LUT_KP + kc) = lo;
        const int oc = k0 + kc - c0;
        if (oc >= 0 && oc < NC) {
          #pragma unroll
          for (int e = 0; e < 8; ++e) own[tok][oc + e] = u[e];
        }
      }
    }
    __syncthreads();
    #pragma unroll
    for (int ks = 0; ks < LUT_KC / 32; ++ks) {
      const int kk = k0 + ks * 32 + lk * 8;
      if (k0 + ks * 32 >= n) break;
      bf16v8 br, bi;
      #pragma unroll
      for (int j = 0; j < 8; ++j) { br[j] = (__bf16)0.0f; bi[j] = (__bf16)0.0f; }
      if (col < n && kk < n) {
        br = *reinterpret_cast<const bf16v8*>(w0 + kk);
        bi = *reinterpret_cast<const bf16v8*>(w1 + kk);
      }
      #pragma unroll
      for (int mt = 0; mt < 4; ++mt) {
        const int at = (mt * 16 + lrow) * LUT_KP + ks * 32 + lk * 8;
        const bf16v8 ah = *reinterpret_cast<const bf16v8*>(uh + at);
        const bf16v8 al = *reinterpret_cast<const bf16v8*>(ul + at);
        acc[0][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, br, acc[0][mt], 0, 0, 0);
        acc[0][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, br, acc[0][mt], 0, 0, 0);
        acc[1][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, bi, acc[1][mt], 0, 0, 0);
        acc[1][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, bi, acc[1][mt], 0, 0, 0);
      }
    }
  }
  // prefixes: the lane's 4 tokens, then the 4 lane groups, then the 16-token tiles
  const lu_channel C = lu_channel_of(A, blk * n + min(col, n - 1));
  float pt = 1.f, qt = 0.f;                          // everything before the 16-token tile
  #pragma unroll
  for (int mt = 0; mt < 4; ++mt) {
    float p[4], q[4];
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int tok = mt * 16 + lk * 4 + r;
      float a = 1.f, bb = 0.f;
      if (tok < nt)
        lu_gate_fast(C, acc[0][mt][r], acc[1][mt][r], own[tok][wave * 16 + lrow], &a, &bb);
      p[r] = r ? a * p[r ? r - 1 : 0] : a;
      q[r] = r ? fmaf(a, q[r ? r - 1 : 0], bb) : bb;
    }
    float pi = p[3], qi = q[3];                      // inclusive over the lane groups
    #pragma unroll
    for (int s = 1; s <= 2; s <<= 1) {
      const float pp = __shfl_up(pi, 16 * s, SM_WAVE), qp = __shfl_up(qi, 16 * s, SM_WAVE);
      if (lk >= s) {
        qi = fmaf(pi, qp, qi);
        pi *= pp;
      }
    }
    float pe = __shfl_up(pi, 16, SM_WAVE), qe = __shfl_up(qi, 16, SM_WAVE);
    if (lk == 0) { pe = 1.f; qe = 0.f; }
    const float pb = pe * pt, qb = fmaf(pe, qt, qe);           // everything before the lane's tokens
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int tok = mt * 16 + lk * 4 + r;
      if (tok < nt && col < n) {
        const int64_t at = (int64_t)(t0 + tok) * A.W + blk * n + col;
        P[at] = p[r] * pb;
        Q[at] = fmaf(p[r], qb, q[r]);
      }
    }
    const float pl = __shfl(pi, 48 + lrow, SM_WAVE), ql = __shfl(qi, 48 + lrow, SM_WAVE);
    qt = fmaf(pl, qt, ql);
    pt *= pl;
  }
}

__global__ __launch_bounds__(64) void linear_unit_carry_kernel(
    const float* __restrict__ P, const float* __restrict__ Q, const int* __restrict__ tiles,
    const int* __restrict__ tile_cu, const int* __restrict__ slots, int W,
    float* __restrict__ state, float* __restrict__ S0) {
  const int b = blockIdx.x, ch = blockIdx.y * 64 + threadIdx.x;
  if (ch >= W) return;
  float* st = state + (int64_t)slots[b] * W + ch;
  float S = *st;
  const int e = tile_cu[b + 1];
  for (int i0 = tile_cu[b]; i0 < e; i0 += 8) {
    float p[8], q[8];
    #pragma unroll
    for (int k = 0; k < 8; ++k) {                    // eight tiles' last prefixes in flight
      const int i = min(i0 + k, e - 1);
      const int64_t at = (int64_t)(tiles[3 * i + 1] + tiles[3 * i + 2] - 1) * W + ch;
      p[k] = P[at];
      q[k] = Q[at];
    }
    #pragma unroll
    for (int k = 0; k < 8; ++k) {
      if (i0 + k < e) {
        S0[(int64_t)(i0 + k) * W + ch] = S;
        S = fmaf(p[k], S, q[k]);
      }
    }
  }
  *st = S;
}

template <int VEC>
__global__ __launch_bounds__(256) void linear_unit_apply_kernel(
    const float* __restrict__ P, const float* __restrict__ Q, const float* __restrict__ S0,
    const int* __restrict__ tiles, const bf16_t* __restrict__ y, int64_t ldp, int W,
    bf16_t* __restrict__ out) {
  const int t0 = tiles[3 * blockIdx.x + 1], nt = tiles[3 * blockIdx.x + 2];
  const int ch = (blockIdx.y * 64 + (threadIdx.x & 63)) * VEC;
  if (ch >= W) return;
  const sm_vec<VEC> s = sm_load<VEC>(S0 + (int64_t)blockIdx.x * W + ch);
  for (int tok = threadIdx.x >> 6; tok < nt; tok += 4) {
    const int64_t at = (int64_t)(t0 + tok) * W + ch;
    const sm_vec<VEC> p = sm_load<VEC>(P + at), q = sm_load<VEC>(Q + at);
    const sm_vec<VEC> yv = sm_load<VEC>(y + (int64_t)(t0 + tok) * ldp + ch);
    sm_vec<VEC> o;
    #pragma unroll
    for (int k = 0; k < VEC; ++k) o.v[k] = fmaf(p.v[k], s.v[k], q.v[k]) * gelu_tanh_f(yv.v[k]);
    sm_store<VEC>(out + at, o);
  }
}

// ---- one token per row. A workgroup takes 16 tokens and 16 channels of a
// block; its four waves share the block's channels as the reduction axis (the
// lane forms its own 8 convolved inputs), partial sums meet in LDS.
template <int TAPS>
__global__ __launch_bounds__(256) void linear_unit_step_kernel(
    const bf16_t* __restrict__ y, const bf16_t* __restrict__ x, const bf16_t* __restrict__ gw,
    int T, lu_args A, float* __restrict__ state, bf16_t* __restrict__ out) {
  __shared__ float red[3][64][8];
  const int t0 = blockIdx.x * 16, blk = blockIdx.y, n = A.n;
  const int tid = threadIdx.x, wave = tid >> 6, l = tid & 63, lrow = l & 15, lk = l >> 4;
  const int keep = A.taps - 1;
  const int ta = min(t0 + lrow, T - 1);              // the lane's A row (repeated past the end)
  const float* tl = A.tails + (int64_t)A.slots[ta] * keep * A.W;
  const bf16_t* xr = x + (int64_t)ta * A.ldp;
  const int col = blockIdx.z * 16 + lrow;
  const bf16_t* w0 = gw + ((int64_t)blk * n + min(col, n - 1)) * n;
  const bf16_t* w1 = w0 + (int64_t)A.W * n;
  f32x4 ar = {0.f, 0.f, 0.f, 0.f}, ai = {0.f, 0.f, 0.f, 0.f};
  for (int ks = wave * 32; ks < n; ks += 128) {      // uniform within a wave
    const int kk = ks + lk * 8;
    float u[8];
    bf16v8 br, bi, hi, lo;
    #pragma unroll
    for (int j = 0; j < 8; ++j) { br[j] = (__bf16)0.0f; bi[j] = (__bf16)0.0f; u[j] = 0.f; }
    if (kk < n) {
      if (col < n) {
        br = *reinterpret_cast<const bf16v8*>(w0 + kk);
        bi = *reinterpret_cast<const bf16v8*>(w1 + kk);
      }
      float wr[TAPS > 0 ? 8 * TAPS : 1];
      if (TAPS > 0) {
        #pragma unroll
        for (int e = 0; e < 8 * TAPS; ++e) wr[e] = A.conv_w[(int64_t)(blk * n + kk) * TAPS + e];
      }
      lu_conv8<TAPS>(A, xr, 0, tl, blk * n + kk, wr, u);
    }
    lu_split(u, &hi, &lo);
    ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, br, ar, 0, 0, 0);
    ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, br, ar, 0, 0, 0);
    ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, bi, ai, 0, 0, 0);
    ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, bi, ai, 0, 0, 0);
  }
  if (wave > 0) {
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      red[wave - 1][l][r] = ar[r];
      red[wave - 1][l][4 + r] = ai[r];
    }
  }
  __syncthreads();
  if (wave > 0 || col >= n) return;
  const int ch = blk * n + col;
  const lu_channel C = lu_channel_of(A, ch);
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = t0 + lk * 4 + r;
    if (t >= T) continue;
    float zr = ar[r], zi = ai[r];
    #pragma unroll
    for (int w = 0; w < 3; ++w) {
      zr += red[w][l][r];
      zi += red[w][l][4 + r];
    }
    const int64_t slot = A.slots[t];
    const float u = lu_conv(A, x + (int64_t)t * A.ldp, 0, A.tails + slot * keep * A.W, ch);
    float a, b;
    lu_gate_fast(C, zr, zi, u, &a, &b);
    float* st = state + slot * A.W + ch;
    const float S = fmaf(a, *st, b);
    *st = S;
    out[(int64_t)t * A.W + ch] = __float2bfloat16(S * gelu_tanh_f(to_f(y[(int64_t)t * A.ldp + ch])));
  }
}

// ---- any size. One workgroup per (token, block): u of the block in LDS, a wave
// per gate output; a and b to memory.
template <typename T>
__global__ __launch_bounds__(256) void linear_unit_plain_kernel(
    const T* __restrict__ x, const T* __restrict__ gw, lu_args A, float* __restrict__ av,
    float* __restrict__ bv) {
  extern __shared__ float lu_u[];                    // [n]
  const int64_t t = blockIdx.x;
  const int blk = blockIdx.y, n = A.n, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int b = A.tok_seq[t], rel = (int)t - A.cu[b];
  const float* tl = A.tails + (int64_t)A.slots[b] * (A.taps - 1) * A.W;
  for (int k = threadIdx.x; k < n; k += 256)
    lu_u[k] = lu_conv(A, x + t * A.ldp, rel, tl, blk * n + k);
  __syncthreads();
  for (int j = wave; j < n; j += 4) {
    const T* w0 = gw + ((int64_t)blk * n + j) * n;
    const T* w1 = w0 + (int64_t)A.W * n;
    float zr = 0.f, zi = 0.f;
    for (int k = lane; k < n; k += 64) {
      zr = fmaf(to_f(w0[k]), lu_u[k], zr);
      zi = fmaf(to_f(w1[k]), lu_u[k], zi);
    }
    zr = sm_wave_sum(zr);
    zi = sm_wave_sum(zi);
    if (lane == 0) {
      float a, bb;
      lu_gate(A, blk * n + j, zr, zi, lu_u[j], &a, &bb);
      av[t * A.W + blk * n + j] = a;
      bv[t * A.W + blk * n + j] = bb;
    }
  }
}
template <typename T>
__global__ __launch_bounds__(64) void linear_unit_walk_kernel(
    const float* __restrict__ av, const float* __restrict__ bv, const T* __restrict__ y, int64_t ldp,
    const int* __restrict__ cu, const int* __restrict__ slots, int W, float* __restrict__ state,
    T* __restrict__ out) {
  const int b = blockIdx.x, ch = blockIdx.y * 64 + threadIdx.x;
  if (ch >= W) return;
  float* st = state + (int64_t)slots[b] * W + ch;
  float S = *st;
  for (int64_t t = cu[b]; t < cu[b + 1]; ++t) {
    S = fmaf(av[t * W + ch], S, bv[t * W + ch]);
    out[t * W + ch] = from_f<T>(S * gelu_tanh_f(to_f(y[t * ldp + ch])));
  }
  *st = S;
}

}  // namespace

// defined in norm_conv.hip
void tap_tail_update(const torch::Tensor& x, int C, torch::Tensor& tails, const torch::Tensor& cu,
                     const torch::Tensor& slots, int taps);

torch::Tensor linear_unit(torch::Tensor proj, torch::Tensor conv_w, torch::Tensor conv_b,
                          torch::Tensor tails, torch::Tensor gates_w, torch::Tensor gates_b,
                          torch::Tensor lam, double c, torch::Tensor state, torch::Tensor cu,
                          torch::Tensor tok_seq, torch::Tensor slots,
                          c10::optional<torch::Tensor> tiles, c10::optional<torch::Tensor> tile_cu) {
  for (const torch::Tensor* t : {&conv_w, &conv_b, &tails, &gates_b, &lam, &state}) {
    SM_CHECK_CUDA(*t); SM_CHECK_F32(*t);
  }
  SM_CHECK_CUDA(gates_w);
  SM_CHECK_CUDA(cu); SM_CHECK_I32(cu); SM_CHECK_CUDA(tok_seq); SM_CHECK_I32(tok_seq);
  SM_CHECK_CUDA(slots); SM_CHECK_I32(slots);
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(1) >= 1 && conv_w.size(1) <= 16,
              "linear_unit: conv weights are [channels, taps], at most 16 taps");
  const int W = conv_w.size(0), taps = conv_w.size(1), B = slots.numel();
  const int64_t T = proj.size(0);
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1 && proj.size(1) >= 2 * (int64_t)W,
              "linear_unit: rows are [y | x]");
  TORCH_CHECK(gates_w.dim() == 4 && gates_w.size(0) == 2 && gates_w.size(2) == gates_w.size(3) &&
              gates_w.size(1) * gates_w.size(2) == W && gates_w.scalar_type() == proj.scalar_type(),
              "linear_unit: gates are [2, blocks, n, n]");
  TORCH_CHECK(conv_b.numel() == W && gates_b.numel() == 2 * (int64_t)W && lam.numel() == W,
              "linear_unit: channel vectors");
  TORCH_CHECK(tails.dim() == 3 && tails.size(1) == taps - 1 && tails.size(2) == W && state.dim() == 2 &&
              state.size(1) == W && cu.numel() == B + 1 && tok_seq.numel() == T,
              "linear_unit: state/batch layout");
  const int blocks = gates_w.size(1), n = gates_w.size(2);
  const bool bf16 = proj.scalar_type() == at::kBFloat16;
  if (!bf16) SM_CHECK_F32(proj);
  auto out = torch::empty({T, (int64_t)W}, proj.options());
  if (T == 0 || B == 0) return out;
  auto stream = at::cuda::getCurrentCUDAStream();
  const lu_args A = {proj.stride(0), W, n, taps, conv_w.data_ptr<float>(), conv_b.data_ptr<float>(),
                     tails.data_ptr<float>(), gates_b.data_ptr<float>(), lam.data_ptr<float>(), (float)c,
                     cu.data_ptr<int>(), tok_seq.data_ptr<int>(), slots.data_ptr<int>()};
  float* sp = state.data_ptr<float>();
  auto f32 = proj.options().dtype(at::kFloat);
  // 16-byte pieces of the x rows and of the gate matrices
  const bool pieces = bf16 && n % 8 == 0 && proj.stride(0) % 8 == 0 &&
                      reinterpret_cast<uintptr_t>(proj.data_ptr()) % 16 == 0;
  if (pieces) {
    const bf16_t* yp = reinterpret_cast<const bf16_t*>(proj.data_ptr());
    const bf16_t* xp = yp + W;
    const bf16_t* gp = reinterpret_cast<const bf16_t*>(gates_w.data_ptr());
    bf16_t* op = reinterpret_cast<bf16_t*>(out.data_ptr());
    if (T == B) {                          // a step's rows are never empty: one token each
      const dim3 grid(SM_CDIV(T, 16), blocks, SM_CDIV(n, 16));
      if (taps == 4)
        linear_unit_step_kernel<4><<<grid, 256, 0, stream>>>(yp, xp, gp, (int)T, A, sp, op);
      else
        linear_unit_step_kernel<0><<<grid, 256, 0, stream>>>(yp, xp, gp, (int)T, A, sp, op);
      SM_CHECK_LAUNCH();
    } else {
      TORCH_CHECK(tiles.has_value() && tile_cu.has_value(), "linear_unit: tiles missing");
      SM_CHECK_CUDA(*tiles); SM_CHECK_I32(*tiles); SM_CHECK_CUDA(*tile_cu); SM_CHECK_I32(*tile_cu);
      TORCH_CHECK(tiles->dim() == 2 && tiles->size(1) == 3 && tiles->size(0) >= 1 &&
                  tile_cu->numel() == B + 1, "linear_unit: tile layout");
      const int nt = tiles->size(0);
      const int* tp = tiles->data_ptr<int>();
      auto P = torch::empty({T, (int64_t)W}, f32), Q = torch::empty({T, (int64_t)W}, f32);
      auto S0 = torch::empty({nt, (int64_t)W}, f32);
#define LU_TILE(TAPS, NW)                                                              \
  linear_unit_tile_kernel<TAPS, NW><<<dim3(nt, blocks, SM_CDIV(n, 16 * NW)), 64 * NW, 0, stream>>>( \
      xp, gp, tp, A, P.data_ptr<float>(), Q.data_ptr<float>())
      if (n <= 64) { if (taps == 4) LU_TILE(4, 4); else LU_TILE(0, 4); }
      else { if (taps == 4) LU_TILE(4, 8); else LU_TILE(0, 8); }
#undef LU_TILE
      SM_CHECK_LAUNCH();
      linear_unit_carry_kernel<<<dim3(B, SM_CDIV(W, 64)), 64, 0, stream>>>(
          P.data_ptr<float>(), Q.data_ptr<float>(), tp, tile_cu->data_ptr<int>(), A.slots, W, sp,
          S0.data_ptr<float>());
      SM_CHECK_LAUNCH();
      linear_unit_apply_kernel<4><<<dim3(nt, SM_CDIV(W, 256)), 256, 0, stream>>>(
          P.data_ptr<float>(), Q.data_ptr<float>(), S0.data_ptr<float>(), tp, yp, proj.stride(0), W, op);
      SM_CHECK_LAUNCH();
    }
  } else {
    TORCH_CHECK(n <= 16384, "linear_unit: blocks of more than 16384 channels");
    auto av = torch::empty({T, (int64_t)W}, f32), bv = torch::empty({T, (int64_t)W}, f32);
#define LU_PLAIN(TY)                                                                           \
  do {                                                                                         \
    const TY* yp = reinterpret_cast<const TY*>(proj.data_ptr());                               \
    linear_unit_plain_kernel<TY><<<dim3(T, blocks), 256, n * sizeof(float), stream>>>(         \
        yp + W, reinterpret_cast<const TY*>(gates_w.data_ptr()), A, av.data_ptr<float>(),      \
        bv.data_ptr<float>());                                                                 \
    SM_CHECK_LAUNCH();                                                                         \
    linear_unit_walk_kernel<TY><<<dim3(B, SM_CDIV(W, 64)), 64, 0, stream>>>(                   \
        av.data_ptr<float>(), bv.data_ptr<float>(), yp, proj.stride(0), A.cu, A.slots, W, sp,  \
        reinterpret_cast<TY*>(out.data_ptr()));                                                \
    SM_CHECK_LAUNCH();                                                                         \
  } while (0)
    if (bf16) LU_PLAIN(bf16_t); else LU_PLAIN(float);
#undef LU_PLAIN
  }
  tap_tail_update(proj.slice(1, W, 2 * (int64_t)W), W, tails, cu, slots, taps);
  return out;
}
