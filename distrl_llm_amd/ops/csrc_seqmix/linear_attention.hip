// Linear attention with a fixed decay per head over a flat varlen batch, fp32
// matrix state per (slot, head):
//   q, k, v = silu of the projection rows;  S <- lambda S + k v^T,  o = S^T q
// then one RMS norm over all heads of a token and a sigmoid gate per entry.
//   linear_attention_chunk  bf16 prompt steps: a workgroup walks a row's tokens
//                           in chunks of 64 on MFMA with the state in its
//                           accumulators
//   linear_attention_scan   fp32 models, steps of few tokens per row, odd sizes:
//                           token by token, state in registers
//   linear_gated_norm       norm over the heads and output gate
// The chunk form, with tokens i, j of a chunk, S the state before it and cnt its
// length:
//   o_i  = lambda^(i+1) S^T q_i + sum_(j<=i) lambda^(i-j) (q_i . k_j) v_j
//   S   <- lambda^cnt S + sum_j k_j (lambda^(cnt-1-j) v_j)^T
// q, k and v are exact in bf16 once rounded after the activation; the fp32
// factors (decayed scores, decayed v, the state) enter the matrix cores as two
// bf16 terms each (x = hi + lo, error <= 2^-17 x) with fp32 accumulation. The
// state is stored value-major ([head][column][key]).
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>
#include "seqmix_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16v8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

namespace {

SM_INLINE float la_silu(float z) { return z * sm_sigmoid(z); }
SM_INLINE __bf16 la_silu_bf16(__bf16 z) {
  const float f = (float)z;
  return (__bf16)(f * sm_fast_sigmoid(f));
}

// ---- token by token. One workgroup per (row, head, 16 value columns): lane
// group of 16 per column, a lane holds the keys 64 i + 4 (lane & 15) .. + 3;
// the dot products over the keys end in lane permutes. Tokens pass through LDS
// in chunks, activated once for the 16 columns.
template <typename T, int NK>
__global__ __launch_bounds__(256) void linear_attention_scan_kernel(
    const T* __restrict__ proj, int64_t ldp, int H, int dk, int vd,
    const float* __restrict__ powers, int np, float* __restrict__ state,
    const int* __restrict__ cu, const int* __restrict__ slots, float* __restrict__ o) {
  constexpr int KP = NK * 64, CH = NK > 4 ? 8 : 16;  // tokens per chunk
  __shared__ __attribute__((aligned(16))) float kb[CH][KP];
  __shared__ __attribute__((aligned(16))) float qb[CH][KP];
  __shared__ float vb[CH][16];
  const int b = blockIdx.x, h = blockIdx.y;
  const int rg = threadIdx.x & 15, cc = threadIdx.x >> 4;
  const int c = blockIdx.z * 16 + cc;
  const int t0 = cu[b], t1 = cu[b + 1];
  if (t1 == t0) return;
  const float lam = powers[h * np + 1];
  const int nq = H * dk;
  float* st = state + (int64_t)slots[b] * H * vd * dk + ((int64_t)h * vd + min(c, vd - 1)) * dk;
  float S[NK][4];
  #pragma unroll
  for (int i = 0; i < NK; ++i)
    #pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int k = 64 * i + 4 * rg + e;
      S[i][e] = (k < dk) ? st[k] : 0.f;
    }
  for (int tc = t0; tc < t1; tc += CH) {
    const int cnt = min(CH, t1 - tc);
    __syncthreads();
    for (int i = threadIdx.x; i < cnt * KP; i += 256) {
      const int t = i / KP, k = i % KP;
      const T* row = proj + (int64_t)(tc + t) * ldp;
      qb[t][k] = (k < dk) ? la_silu(to_f(row[h * dk + k])) : 0.f;
      kb[t][k] = (k < dk) ? la_silu(to_f(row[nq + h * dk + k])) : 0.f;
    }
    for (int i = threadIdx.x; i < cnt * 16; i += 256) {
      const int t = i / 16, col = blockIdx.z * 16 + i % 16;
      vb[t][i % 16] = (col < vd)
          ? la_silu(to_f(proj[(int64_t)(tc + t) * ldp + 2 * nq + h * vd + col])) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < cnt; ++t) {
      const float v = vb[t][cc];
      float acc = 0.f;
      #pragma unroll
      for (int i = 0; i < NK; ++i) {
        const float4 k4 = *reinterpret_cast<const float4*>(&kb[t][64 * i + 4 * rg]);
        const float4 q4 = *reinterpret_cast<const float4*>(&qb[t][64 * i + 4 * rg]);
        const float kk[4] = {k4.x, k4.y, k4.z, k4.w}, qq[4] = {q4.x, q4.y, q4.z, q4.w};
        #pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[i][e] = fmaf(lam, S[i][e], kk[e] * v);
          acc = fmaf(qq[e], S[i][e], acc);
        }
      }
      acc = sm_row16_sum(acc);
      if (rg == 0 && c < vd) o[((int64_t)(tc + t) * H + h) * vd + c] = acc;
    }
  }
  if (c >= vd) return;
  #pragma unroll
  for (int i = 0; i < NK; ++i)
    #pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int k = 64 * i + 4 * rg + e;
      if (k < dk) st[k] = S[i][e];
    }
}

// ---- chunks of 64 tokens. One workgroup (4 waves) per (row, head, 32 value
// columns); wave w owns the queries 16 w .. of a chunk and the 16-key tiles w,
// w + 4, ... of the state. Rows are the slowest grid axis: rows of a few tokens
// beside long ones then leave the chip evenly filled. KS: 32-entry steps of the key axis (dk <= 32 KS).
// MFMA 16x16x32 bf16 fragments: A lane l -> row l & 15, k (l >> 4) * 8 ..;
// B lane l -> column l & 15, same k; D lane l reg r -> row (l >> 4) * 4 + r,
// column l & 15.
#define LAC 64          // tokens per chunk
#define LAC_V 32        // value columns per workgroup
#define LAC_TP (LAC + 8)    // LDS pitch of token-contiguous rows (bf16)
#define LAC_PP 36           // LDS pitch of the score tile (floats)
SM_INLINE void la_split(float x, __bf16* hi, __bf16* lo) {
  *hi = (__bf16)x;
  *lo = (__bf16)(x - (float)*hi);
}
template <int KS>
constexpr size_t lac_lds_bytes() {
  return ((size_t)LAC * (KS * 32 + 8) + (size_t)KS * 32 * LAC_TP + 3 * LAC_V * LAC_TP +
          2 * (size_t)LAC_V * (KS * 32 + 8)) * 2 + (4 * 16 * LAC_PP + LAC + 4) * 4;
}
template <int KS>
__global__ __launch_bounds__(256, 2) void linear_attention_chunk_kernel(
    const bf16_t* __restrict__ proj, int64_t ldp, int H, int dk, int vd,
    const float* __restrict__ powers, int np, float* __restrict__ state,
    const int* __restrict__ cu, const int* __restrict__ slots, float* __restrict__ o) {
  constexpr int DP = KS * 32, KPT = DP + 8, MI = (KS + 1) / 2;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  __bf16* k_lds = reinterpret_cast<__bf16*>(smem);        // [LAC][KPT]
  __bf16* kT = k_lds + LAC * KPT;                         // [DP][LAC_TP]
  __bf16* vT = kT + DP * LAC_TP;                          // [LAC_V][LAC_TP]
  __bf16* vh = vT + LAC_V * LAC_TP;                       // decayed v, hi and lo terms
  __bf16* vl = vh + LAC_V * LAC_TP;
  __bf16* sh = vl + LAC_V * LAC_TP;                       // [LAC_V][KPT] state, hi and lo
  __bf16* sl = sh + LAC_V * KPT;
  float* p_all = reinterpret_cast<float*>(sl + LAC_V * KPT);      // [4][16][LAC_PP]
  float* pw = p_all + 4 * 16 * LAC_PP;                            // [LAC + 1] powers of the decay
  const int h = blockIdx.x, v0 = blockIdx.y * LAC_V, b = blockIdx.z;
  const int tid = threadIdx.x, wave = tid >> 6, l = tid & 63, lrow = l & 15, lk = l >> 4;
  const int t0 = cu[b], n = cu[b + 1] - t0;
  if (n == 0) return;
  if (tid <= LAC) pw[tid] = powers[h * np + tid];
  const int nq = H * dk;
  float* st = state + (int64_t)slots[b] * H * vd * dk + (int64_t)h * vd * dk;
  float* p_lds = p_all + wave * 16 * LAC_PP;

  // state tiles: rows = keys, columns = values
  f32x4 sacc[MI][2];
  #pragma unroll
  for (int mi = 0; mi < MI; ++mi)
    #pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      const int k = (wave + 4 * mi) * 16 + lk * 4, c = v0 + nt * 16 + lrow;
      sacc[mi][nt] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (k < dk && c < vd) sacc[mi][nt] = *reinterpret_cast<const f32x4*>(st + (int64_t)c * dk + k);
    }

  // a chunk's projection rows, fetched into registers one chunk ahead: the
  // thread's pieces of k and v, the lane's queries as A fragments
  constexpr int KI = LAC * (DP / 8) / 256;
  bf16v8 kraw[KI], vraw, qraw[KS], zero;
  #pragma unroll
  for (int j = 0; j < 8; ++j) zero[j] = (__bf16)0.0f;
  const int vtok = tid % LAC, vc = (tid / LAC) * 8;
  auto fetch = [&](int c0) {
    const int cnt = min(LAC, n - c0);
    const bf16_t* base = proj + (int64_t)(t0 + c0) * ldp;
    #pragma unroll
    for (int i = 0; i < KI; ++i) {
      const int tok = (i * 256 + tid) % LAC, c = (i * 256 + tid) / LAC * 8;
      kraw[i] = zero;
      if (tok < cnt && c < dk)
        kraw[i] = *reinterpret_cast<const bf16v8*>(base + (int64_t)tok * ldp + nq + h * dk + c);
    }
    vraw = zero;
    if (vtok < cnt && v0 + vc < vd)
      vraw = *reinterpret_cast<const bf16v8*>(base + (int64_t)vtok * ldp + 2 * nq + h * vd + v0 + vc);
    const int qi = wave * 16 + lrow;
    #pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int c = ks * 32 + lk * 8;
      qraw[ks] = zero;
      if (qi < cnt && c < dk)
        qraw[ks] = *reinterpret_cast<const bf16v8*>(base + (int64_t)qi * ldp + h * dk + c);
    }
  };
  fetch(0);

  for (int c0 = 0; c0 < n; c0 += LAC) {
    const int cnt = min(LAC, n - c0);
    __syncthreads();                               // the previous chunk's LDS reads are done
    // keys, activated (silu(0) = 0: padding stays zero), token-major and key-major
    #pragma unroll
    for (int i = 0; i < KI; ++i) {
      const int tok = (i * 256 + tid) % LAC, c = (i * 256 + tid) / LAC * 8;
      bf16v8 kv;
      #pragma unroll
      for (int j = 0; j < 8; ++j) kv[j] = la_silu_bf16(kraw[i][j]);
      *reinterpret_cast<bf16v8*>(k_lds + tok * KPT + c) = kv;
      #pragma unroll
      for (int j = 0; j < 8; ++j) kT[(c + j) * LAC_TP + tok] = kv[j];
    }
    // values, activated, as they are and decayed to the chunk's end
    {
      const float dec = (vtok < cnt) ? pw[cnt - 1 - vtok] : 0.f;
      #pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int at = (vc + j) * LAC_TP + vtok;
        const __bf16 v = la_silu_bf16(vraw[j]);
        vT[at] = v;
        __bf16 hi, lo;
        la_split((float)v * dec, &hi, &lo);
        vh[at] = hi;
        vl[at] = lo;
      }
    }
    // the state before the chunk, [column][key], four keys per store
    #pragma unroll
    for (int mi = 0; mi < MI; ++mi) {
      const int k = (wave + 4 * mi) * 16 + lk * 4;
      if (k < DP) {
        #pragma unroll
        for (int nt = 0; nt < 2; ++nt) {
          union { __bf16 e[4]; uint2 u; } hi, lo;
          #pragma unroll
          for (int r = 0; r < 4; ++r) la_split(sacc[mi][nt][r], &hi.e[r], &lo.e[r]);
          *reinterpret_cast<uint2*>(sh + (nt * 16 + lrow) * KPT + k) = hi.u;
          *reinterpret_cast<uint2*>(sl + (nt * 16 + lrow) * KPT + k) = lo.u;
        }
      }
    }
    bf16v8 qf[KS];
    #pragma unroll
    for (int ks = 0; ks < KS; ++ks)
      #pragma unroll
      for (int j = 0; j < 8; ++j) qf[ks][j] = la_silu_bf16(qraw[ks][j]);
    __syncthreads();
    if (c0 + LAC < n) fetch(c0 + LAC);             // lands while this chunk is computed
    if (wave * 16 < cnt) {
      // what the state before the chunk gives
      f32x4 acc[2];
      #pragma unroll
      for (int nt = 0; nt < 2; ++nt) {
        acc[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
        #pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          const int at = (nt * 16 + lrow) * KPT + ks * 32 + lk * 8;
          acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              qf[ks], *reinterpret_cast<const bf16v8*>(sh + at), acc[nt], 0, 0, 0);
          acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              qf[ks], *reinterpret_cast<const bf16v8*>(sl + at), acc[nt], 0, 0, 0);
        }
        #pragma unroll
        for (int r = 0; r < 4; ++r) acc[nt][r] *= pw[wave * 16 + lk * 4 + r + 1];
      }
      // the chunk's own keys, 32 at a time; those after the wave's last query
      // count for nothing
      #pragma unroll
      for (int half = 0; half < 2; ++half) {
        if (half * 32 > wave * 16 + 15) break;
        #pragma unroll
        for (int ct = 0; ct < 2; ++ct) {
          f32x4 s = {0.f, 0.f, 0.f, 0.f};
          const int j = half * 32 + ct * 16 + lrow;
          #pragma unroll
          for (int ks = 0; ks < KS; ++ks)
            s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                qf[ks], *reinterpret_cast<const bf16v8*>(k_lds + j * KPT + ks * 32 + lk * 8), s, 0, 0, 0);
          #pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int i = wave * 16 + lk * 4 + r;
            p_lds[(lk * 4 + r) * LAC_PP + ct * 16 + lrow] = (j <= i) ? s[r] * pw[i - j] : 0.f;
          }
        }
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_s_waitcnt(0xc07f);        // the wave's LDS writes have landed
        const float4 w0 = *reinterpret_cast<const float4*>(p_lds + lrow * LAC_PP + lk * 8);
        const float4 w1 = *reinterpret_cast<const float4*>(p_lds + lrow * LAC_PP + lk * 8 + 4);
        const float pv[8] = {w0.x, w0.y, w0.z, w0.w, w1.x, w1.y, w1.z, w1.w};
        bf16v8 ph, pl;
        #pragma unroll
        for (int j = 0; j < 8; ++j) {
          __bf16 hi, lo;
          la_split(pv[j], &hi, &lo);
          ph[j] = hi;
          pl[j] = lo;
        }
        #pragma unroll
        for (int nt = 0; nt < 2; ++nt) {
          const bf16v8 vf = *reinterpret_cast<const bf16v8*>(
              vT + (nt * 16 + lrow) * LAC_TP + half * 32 + lk * 8);
          acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph, vf, acc[nt], 0, 0, 0);
          acc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, vf, acc[nt], 0, 0, 0);
        }
        __builtin_amdgcn_wave_barrier();           // p_lds is rewritten by the next half
      }
      #pragma unroll
      for (int nt = 0; nt < 2; ++nt) {
        const int c = v0 + nt * 16 + lrow;
        #pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int i = wave * 16 + lk * 4 + r;
          if (i < cnt && c < vd) o[((int64_t)(t0 + c0 + i) * H + h) * vd + c] = acc[nt][r];
        }
      }
    }
    // the state after the chunk
    const float full = pw[cnt];
    #pragma unroll
    for (int mi = 0; mi < MI; ++mi) {
      const int k = (wave + 4 * mi) * 16;
      if (k < DP) {
        #pragma unroll
        for (int nt = 0; nt < 2; ++nt) sacc[mi][nt] *= full;
        #pragma unroll
        for (int ks = 0; ks < LAC / 32; ++ks) {
          const bf16v8 kf = *reinterpret_cast<const bf16v8*>(kT + (k + lrow) * LAC_TP + ks * 32 + lk * 8);
          #pragma unroll
          for (int nt = 0; nt < 2; ++nt) {
            const int at = (nt * 16 + lrow) * LAC_TP + ks * 32 + lk * 8;
            sacc[mi][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                kf, *reinterpret_cast<const bf16v8*>(vh + at), sacc[mi][nt], 0, 0, 0);
            sacc[mi][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                kf, *reinterpret_cast<const bf16v8*>(vl + at), sacc[mi][nt], 0, 0, 0);
          }
        }
      }
    }
  }
  #pragma unroll
  for (int mi = 0; mi < MI; ++mi)
    #pragma unroll
    for (int nt = 0; nt < 2; ++nt) {
      const int k = (wave + 4 * mi) * 16 + lk * 4, c = v0 + nt * 16 + lrow;
      if (k < dk && c < vd) *reinterpret_cast<f32x4*>(st + (int64_t)c * dk + k) = sacc[mi][nt];
    }
}

// out = o / rms(o) * w * sigmoid(gate), the mean over the whole row of nv
// entries; gate rows are ldg apart.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void linear_gated_norm_kernel(
    const float* __restrict__ o, const float* __restrict__ w, const T* __restrict__ gate,
    int64_t ldg, float eps, int nv, T* __restrict__ out) {
  __shared__ float red[4];
  const int64_t t = blockIdx.x;
  const float* orow = o + t * nv;
  float ss = 0.f;
  for (int d = threadIdx.x * VEC; d < nv; d += blockDim.x * VEC) {
    const sm_vec<VEC> v = sm_load<VEC>(orow + d);
    #pragma unroll
    for (int k = 0; k < VEC; ++k) ss += v.v[k] * v.v[k];
  }
  const float inv = 1.0f / sqrtf(sm_block_sum(ss, red) / (float)nv + eps);
  for (int d = threadIdx.x * VEC; d < nv; d += blockDim.x * VEC) {
    sm_vec<VEC> v = sm_load<VEC>(orow + d);
    const sm_vec<VEC> wv = sm_load<VEC>(w + d), g = sm_load<VEC>(gate + t * ldg + d);
    #pragma unroll
    for (int k = 0; k < VEC; ++k) v.v[k] = v.v[k] * inv * wv.v[k] * sm_sigmoid(g.v[k]);
    sm_store<VEC>(out + t * nv + d, v);
  }
}

template <int KS>
void launch_chunk(dim3 grid, hipStream_t stream, const bf16_t* proj, int64_t ldp, int H, int dk,
                  int vd, const float* powers, int np, float* state, const int* cu,
                  const int* slots, float* o) {
  auto kern = linear_attention_chunk_kernel<KS>;
  constexpr size_t lds = lac_lds_bytes<KS>();
  static bool raised = false;        // once, not under a later graph capture
  if (lds > 64 * 1024 && !raised) {
    TORCH_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(kern),
                                    hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess,
                "linear attention: cannot raise the LDS limit");
    raised = true;
  }
  kern<<<grid, 256, lds, stream>>>(proj, ldp, H, dk, vd, powers, np, state, cu, slots, o);
}

}  // namespace

torch::Tensor linear_attention(torch::Tensor proj, int64_t heads, int64_t dim, int64_t vdim,
                               torch::Tensor powers, torch::Tensor norm_w, double eps,
                               torch::Tensor state, torch::Tensor cu, torch::Tensor slots,
                               int64_t max_tile) {
  SM_CHECK_CUDA(powers); SM_CHECK_F32(powers); SM_CHECK_CUDA(norm_w); SM_CHECK_F32(norm_w);
  SM_CHECK_CUDA(state); SM_CHECK_F32(state); SM_CHECK_CUDA(cu); SM_CHECK_I32(cu);
  SM_CHECK_CUDA(slots); SM_CHECK_I32(slots);
  const int64_t T = proj.size(0);
  const int H = heads, dk = dim, vd = vdim, B = slots.numel();
  const int nq = H * dk, nv = H * vd;
  TORCH_CHECK(B <= 65535, "linear_attention: more than 65535 rows in a step");
  TORCH_CHECK(H >= 1 && dk >= 1 && vd >= 1 && dk <= 512, "linear_attention: key size above 512");
  TORCH_CHECK(proj.is_cuda() && proj.dim() == 2 && proj.stride(1) == 1 &&
              proj.size(1) >= 2 * (int64_t)nq + 2 * nv, "linear_attention: rows are [q | k | v | gate]");
  TORCH_CHECK(powers.dim() == 2 && powers.size(0) == H && powers.size(1) > LAC,
              "linear_attention: powers 0 .. 64 of every head's decay");
  TORCH_CHECK(norm_w.numel() == nv, "linear_attention: norm weight");
  TORCH_CHECK(state.dim() == 2 && state.size(1) == (int64_t)nv * dk && cu.numel() == B + 1,
              "linear_attention: state/batch layout");
  const bool bf16 = proj.scalar_type() == at::kBFloat16;
  if (!bf16) SM_CHECK_F32(proj);
  auto out = torch::empty({T, (int64_t)nv}, proj.options());
  if (T == 0 || B == 0) return out;
  auto o = torch::empty({T, (int64_t)nv}, proj.options().dtype(at::kFloat));
  auto stream = at::cuda::getCurrentCUDAStream();
  const int64_t ldp = proj.stride(0);
  const int np = powers.size(1);
  const float* pp = powers.data_ptr<float>();
  float* sp = state.data_ptr<float>();
  float* op = o.data_ptr<float>();
  const int* cp = cu.data_ptr<int>();
  const int* sl = slots.data_ptr<int>();
  // 16-byte pieces of the projection rows
  const bool chunked = bf16 && max_tile > 4 && dk % 8 == 0 && vd % 8 == 0 && dk <= 256 &&
                       ldp % 8 == 0 && reinterpret_cast<uintptr_t>(proj.data_ptr()) % 16 == 0;
  if (chunked) {
    const bf16_t* xp = reinterpret_cast<const bf16_t*>(proj.data_ptr());
    const dim3 grid(H, SM_CDIV(vd, LAC_V), B);
    if (dk <= 64) launch_chunk<2>(grid, stream, xp, ldp, H, dk, vd, pp, np, sp, cp, sl, op);
    else if (dk <= 128) launch_chunk<4>(grid, stream, xp, ldp, H, dk, vd, pp, np, sp, cp, sl, op);
    else launch_chunk<8>(grid, stream, xp, ldp, H, dk, vd, pp, np, sp, cp, sl, op);
  } else {
    const dim3 grid(B, H, SM_CDIV(vd, 16));
#define LA_SCAN(TY, NK)                                                              \
  linear_attention_scan_kernel<TY, NK><<<grid, 256, 0, stream>>>(                    \
      reinterpret_cast<const TY*>(proj.data_ptr()), ldp, H, dk, vd, pp, np, sp, cp, sl, op)
#define LA_SCAN_K(TY)                                                                \
  do {                                                                               \
    if (dk <= 64) LA_SCAN(TY, 1); else if (dk <= 128) LA_SCAN(TY, 2);                \
    else if (dk <= 192) LA_SCAN(TY, 3); else if (dk <= 256) LA_SCAN(TY, 4);          \
    else LA_SCAN(TY, 8);                                                             \
  } while (0)
    if (bf16) LA_SCAN_K(bf16_t); else LA_SCAN_K(float);
#undef LA_SCAN_K
#undef LA_SCAN
  }
  SM_CHECK_LAUNCH();
  const int64_t g0 = 2 * (int64_t)nq + nv;
  const int64_t esz = bf16 ? 2 : 4;
  const bool vec = nv % 4 == 0 && ldp % 4 == 0 &&
                   (reinterpret_cast<uintptr_t>(proj.data_ptr()) + g0 * esz) % (4 * esz) == 0;
#define LA_NORM(TY, VEC)                                                             \
  linear_gated_norm_kernel<TY, VEC><<<T, 256, 0, stream>>>(                          \
      op, norm_w.data_ptr<float>(), reinterpret_cast<const TY*>(proj.data_ptr()) + g0, ldp, \
      (float)eps, nv, reinterpret_cast<TY*>(out.data_ptr()))
  if (bf16) { if (vec) LA_NORM(bf16_t, 4); else LA_NORM(bf16_t, 1); }
  else { if (vec) LA_NORM(float, 4); else LA_NORM(float, 1); }
#undef LA_NORM
  SM_CHECK_LAUNCH();
  return out;
}
