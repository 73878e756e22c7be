// Tiled MFMA form of the windowed softmax attention for bf16 prompt portions.
//
// One workgroup (4 waves) per (tile of <= 64 consecutive queries of one
// sequence, query head); wave w owns queries 16 w .. 16 w + 15: their scores,
// their online softmax and their value sums. The keys a tile can see are one
// list: the kept first tokens that lie before the window of the tile's first
// query, then everything from that window's start to the tile's last query;
// the list is walked in blocks of KB keys (64; 32 for the wide key rows of
// folded queries, so that more than one workgroup fits a CU) whose key columns
// (the head's kv head, or the whole key row for folded queries) and V rows
// (transposed) are staged in LDS once per tile.
//   scores   MFMA 16x16x32: A = the wave's queries (registers, loaded once),
//            B = K rows from LDS
//   softmax  fp32 in the MFMA's result layout; cap, distance bias and mask per
//            score, the sink where the sum is closed; row reductions over the 16 lanes of a row by lane
//            permutes. The distance bias depends on (head, distance) only and
//            a wave's 16 queries meet a block's keys at KB + 15 distances:
//            the wave tabulates those once per block instead of taking a
//            logarithm per score
//   values   the fp32 weights go through a wave-private LDS tile to the A
//            layout and are split into two bf16 terms (p = hi + lo, error
//            <= 2^-17 p); B = V^T from LDS; fp32 accumulation
// Two maps (differential attention): a block's key columns of both maps are
// staged together; each map's scores and softmax are taken in turn, its weights
// wait in registers as A fragments, and every V fragment is read from LDS once
// for both. Where the softmaxes are closed, the difference of the two results
// and its norm over the head's values are formed in the result layout (a row's
// values lie in 16 lanes).
// The output gate's sigmoid (per head or per entry) multiplies the row there.
#include <torch/extension.h>
#include <ATen/cuda/CUDAContext.h>
#include "seqmix_common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16v8;
typedef __attribute__((ext_vector_type(4))) float f32x4;

namespace {

// cap tanh(x / cap), tanh z = 1 - 2 / (1 + e^(2z)): absolute error of a few
// fp32 roundings of cap; saturates to +-cap. ic2 = 2 / cap.
SM_INLINE float wam_cap(float x, float cap, float ic2) {
  return fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(1.0f + __expf(x * ic2)), cap);
}

// NT: 16-column value tiles per wave (vd <= 16 NT); KS: 32-entry steps of the
// query/key dot product held in registers (KD <= 32 KS); KB: keys per block;
// DIST: the distance bias is taken off the scores (r1, r2 given); MAPS: query
// and key maps per head; EXT: chunks and capped scores (without it the view is a
// window at most, which costs the register-bound variants nothing).
template <int NT, int KS, int KB, bool DIST, int MAPS, bool EXT>
__global__ __launch_bounds__(256, 2) void window_attention_mfma_kernel(
    const bf16_t* __restrict__ q, int KD,  // [Tn, H MAPS, KD]
    const bf16_t* __restrict__ cache,      // [rows, G (MAPS dk + vd)]
    const int* __restrict__ block_tables, int max_nb, int block_size,
    const int* __restrict__ positions,
    const int* __restrict__ tiles,         // [ntiles, 3] = (batch row, first token, queries)
    int H, int G, int dk, int vd, int whole_key, float scale, wa_view vw,
    const float* __restrict__ r1, const float* __restrict__ r2,
    const bf16_t* __restrict__ gate, int64_t ldg, int gs, wa_diff df,
    bf16_t* __restrict__ out) {            // [Tn, H vd]
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  const int ksteps = (KD + 31) / 32;
  const int KP = MAPS * ksteps * 32 + 8;           // k_lds row pitch (bf16)
  const int NVp = (vd + 15) / 16 * 16;
  constexpr int WAM_KB = KB;
  constexpr int WAM_VP = KB + 8;                   // v_lds row pitch (bf16)
  constexpr int WAM_PP = KB + 4;                   // p_lds row pitch (floats)
  constexpr int WAM_TB = KB + 16;                  // distance-bias table per wave
  bf16_t* k_lds = reinterpret_cast<bf16_t*>(smem);                 // [KB][KP]
  bf16_t* v_lds = k_lds + WAM_KB * KP;                             // [NVp][WAM_VP]
  float* p_all = reinterpret_cast<float*>(v_lds + NVp * WAM_VP);   // [4][16][WAM_PP]
  int* krow = reinterpret_cast<int*>(p_all + 4 * 16 * WAM_PP);     // [KB]
  float* tb_all = reinterpret_cast<float*>(krow + KB);             // [4][WAM_TB], DIST only

  const int tile = blockIdx.x, hd = blockIdx.y;
  const int b = tiles[3 * tile], t0 = tiles[3 * tile + 1], nq = tiles[3 * tile + 2];
  const int tid = threadIdx.x, l = tid & 63, lrow = l & 15, lk = l >> 4;
  const int wave = tid >> 6;
  const int W = G * (MAPS * dk + vd);
  const int grp = hd / (H / G);
  const int koff = whole_key ? 0 : grp * MAPS * dk, voff = G * MAPS * dk + grp * vd;
  const int p0 = positions[t0], plast = p0 + nq - 1;
  const int lo = wa_first(vw, p0);
  const int nf = min(vw.keep, lo);                 // kept keys before the first window or chunk
  const int n = nf + (plast - lo + 1);             // keys in the tile's list
  const int nblk = (n + WAM_KB - 1) / WAM_KB;
  const int* bt = block_tables + (int64_t)b * max_nb;
  float* p_lds = p_all + wave * 16 * WAM_PP;
  float* tb = tb_all + wave * WAM_TB;
  const bool active = wave * 16 < nq;
  const float ic2 = (EXT && vw.cap > 0.f) ? 2.0f / vw.cap : 0.f;
  const float a1 = DIST ? r1[hd] : 0.f, a2 = DIST ? r2[hd] : 0.f;

  // the wave's queries as A fragments: row lrow, k = ks * 32 + lk * 8 ..
  bf16v8 qf[MAPS][KS];
  #pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) {
    const int qi = wave * 16 + lrow;
    const bf16_t* qp = q + (((int64_t)(t0 + min(qi, nq - 1)) * H + hd) * MAPS + mp) * KD;
    #pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      #pragma unroll
      for (int j = 0; j < 8; ++j) qf[mp][ks][j] = (__bf16)0.0f;
      const int kk = ks * 32 + lk * 8;
      if (ks < ksteps && qi < nq && kk < KD) qf[mp][ks] = *reinterpret_cast<const bf16v8*>(qp + kk);
    }
  }
  // padding rows of v_lds (value columns vd .. NVp) stay zero
  for (int i = tid; i < (NVp - vd) * WAM_VP; i += 256) v_lds[vd * WAM_VP + i] = __float2bfloat16(0.f);

  int first[EXT ? 4 : 1];                          // where each of the lane's queries starts to see
  #pragma unroll
  for (int r = 0; r < 4 && EXT; ++r)
    first[r] = wa_first(vw, p0 + min(wave * 16 + lk * 4 + r, nq - 1));
  float m[MAPS][4], lsum[MAPS][4];
  f32x4 acc[MAPS][NT];
  #pragma unroll
  for (int mp = 0; mp < MAPS; ++mp) {
    #pragma unroll
    for (int r = 0; r < 4; ++r) { m[mp][r] = -INFINITY; lsum[mp][r] = 0.f; }
    #pragma unroll
    for (int i = 0; i < NT; ++i) acc[mp][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  for (int kb = 0; kb < nblk; ++kb) {
    const int i0 = kb * WAM_KB;
    __syncthreads();                               // the previous block's LDS reads are done
    if (tid < WAM_KB) {
      const int i = min(i0 + tid, n - 1);          // list entries past the end are masked below
      const int j = (i < nf) ? i : lo + (i - nf);
      krow[tid] = bt[j / block_size] * block_size + j % block_size;
    }
    __syncthreads();
    // key columns: [key][map][KD], zero beyond KD
    const int pieces = MAPS * ksteps * 4;
    for (int i = tid; i < WAM_KB * pieces; i += 256) {
      const int key = i / pieces, cc = i % pieces;
      const int mp = (MAPS > 1 && cc >= ksteps * 4) ? 1 : 0;
      const int c = (cc - mp * ksteps * 4) * 8;
      bf16v8 v;
      if (c < KD) {
        v = *reinterpret_cast<const bf16v8*>(cache + (int64_t)krow[key] * W + koff + mp * dk + c);
      } else {
        #pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = (__bf16)0.0f;
      }
      *reinterpret_cast<bf16v8*>(k_lds + key * KP + cc * 8) = v;
    }
    // V rows, transposed: v_lds[column][key]
    for (int i = tid; i < WAM_KB * (vd / 8); i += 256) {
      const int key = i % WAM_KB, c = (i / WAM_KB) * 8;
      const bf16v8 v = *reinterpret_cast<const bf16v8*>(cache + (int64_t)krow[key] * W + voff + c);
      #pragma unroll
      for (int j = 0; j < 8; ++j)
        *reinterpret_cast<__bf16*>(v_lds + (c + j) * WAM_VP + key) = v[j];
    }
    __syncthreads();
    if (!active) continue;
    // a block of the window part that starts after the wave's last query, or
    // ends before the window of its first query, holds nothing the wave sees
    if (i0 >= nf) {
      const int jb0 = lo + (i0 - nf);
      const int wq_last = min(plast, p0 + wave * 16 + 15), wq_first = p0 + wave * 16;
      if (jb0 > wq_last) continue;
      if (EXT) {
        if (jb0 + WAM_KB - 1 < wa_first(vw, wq_first) && jb0 >= vw.keep) continue;
      } else if (vw.window > 0 && jb0 + WAM_KB - 1 < wq_first - vw.window + 1 && jb0 >= vw.keep) {
        continue;
      }
    }

    // distance bias of this wave and block: the block's keys are consecutive
    // positions jb0 .. jb0 + KB - 1 once the list is past the kept tokens, and
    // tb[(query - 16 wave) + (KB - 1 - key column)] covers every pair
    const bool tabled = DIST && i0 >= nf;
    if (DIST && tabled) {
      const int dbase = p0 + wave * 16 - (lo + (i0 - nf)) - (KB - 1);
      for (int i = l; i < KB + 15; i += 64)
        tb[i] = a1 * log1pf(a2 * (float)max(dbase + i, 0));
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_s_waitcnt(0xc07f);
    }

    float cr[MAPS][4];
    bf16v8 a_hi[MAPS][KB / 32], a_lo[MAPS][KB / 32];
    #pragma unroll
    for (int mp = 0; mp < MAPS; ++mp) {
      f32x4 s[KB / 16];
      #pragma unroll
      for (int ct = 0; ct < KB / 16; ++ct) {
        s[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
        #pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          if (ks < ksteps) {
            const bf16v8 kf = *reinterpret_cast<const bf16v8*>(
                k_lds + (ct * 16 + lrow) * KP + (mp * ksteps + ks) * 32 + lk * 8);
            s[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[mp][ks], kf, s[ct], 0, 0, 0);
          }
        }
      }
      // result layout: reg r -> query lk * 4 + r, lane column lrow -> key ct * 16 + lrow
      #pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int qi = wave * 16 + lk * 4 + r;
        const int prow = (qi < nq) ? p0 + qi : -1;
        float sv[KB / 16];
        float bm = -INFINITY;
        #pragma unroll
        for (int ct = 0; ct < KB / 16; ++ct) {
          const int i = i0 + ct * 16 + lrow;
          const int j = (i < nf) ? i : lo + (i - nf);
          const bool in = EXT ? j >= first[EXT ? r : 0] : vw.window <= 0 || prow - j < vw.window;
          const bool seen = i < n && j <= prow && (in || j < vw.keep);
          float x = s[ct][r] * scale;
          if (EXT) x = (ic2 > 0.f) ? wam_cap(x, vw.cap, ic2) : x;
          if (DIST) {
            if (tabled) x -= tb[lk * 4 + r + (KB - 1) - (ct * 16 + lrow)];
            else if (seen) x -= a1 * log1pf(a2 * (float)(prow - j));
          }
          sv[ct] = seen ? x : -INFINITY;
          bm = fmaxf(bm, sv[ct]);
        }
        bm = sm_row16_max(bm);
        const float mn = fmaxf(m[mp][r], bm);
        const float c = (mn == -INFINITY) ? 1.0f : expf(m[mp][r] - mn);
        float ps = 0.f;
        #pragma unroll
        for (int ct = 0; ct < KB / 16; ++ct) {
          const float pv = (sv[ct] == -INFINITY) ? 0.f : expf(sv[ct] - mn);
          ps += pv;
          p_lds[(lk * 4 + r) * WAM_PP + ct * 16 + lrow] = pv;
        }
        ps = sm_row16_sum(ps);
        lsum[mp][r] = lsum[mp][r] * c + ps;
        m[mp][r] = mn;
        cr[mp][r] = c;
      }
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_s_waitcnt(0xc07f);
      // weights as A fragments: row lrow, keys ks2 * 32 + lk * 8 ..
      #pragma unroll
      for (int ks2 = 0; ks2 < KB / 32; ++ks2) {
        const float4 w0 = *reinterpret_cast<const float4*>(p_lds + lrow * WAM_PP + ks2 * 32 + lk * 8);
        const float4 w1 = *reinterpret_cast<const float4*>(p_lds + lrow * WAM_PP + ks2 * 32 + lk * 8 + 4);
        const float pv[8] = {w0.x, w0.y, w0.z, w0.w, w1.x, w1.y, w1.z, w1.w};
        #pragma unroll
        for (int j = 0; j < 8; ++j) {
          const __bf16 hi = (__bf16)pv[j];
          a_hi[mp][ks2][j] = hi;
          a_lo[mp][ks2][j] = (__bf16)(pv[j] - (float)hi);
        }
      }
      __builtin_amdgcn_wave_barrier();             // p_lds is rewritten by the next map or block
    }
    #pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      if (nt * 16 < vd) {
        #pragma unroll
        for (int mp = 0; mp < MAPS; ++mp)
          #pragma unroll
          for (int r = 0; r < 4; ++r) acc[mp][nt][r] *= cr[mp][r];
        #pragma unroll
        for (int ks2 = 0; ks2 < KB / 32; ++ks2) {
          const bf16v8 vf = *reinterpret_cast<const bf16v8*>(
              v_lds + (nt * 16 + lrow) * WAM_VP + ks2 * 32 + lk * 8);
          #pragma unroll
          for (int mp = 0; mp < MAPS; ++mp) {
            acc[mp][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_hi[mp][ks2], vf, acc[mp][nt], 0, 0, 0);
            acc[mp][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a_lo[mp][ks2], vf, acc[mp][nt], 0, 0, 0);
          }
        }
      }
    }
  }

  if (!active) return;
  const float lam = (MAPS == 2) ? wa_lambda(df, dk, l) : 0.f;
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int qi = wave * 16 + lk * 4 + r;
    float f = 1.0f / (lsum[0][r] + wa_sink(vw, hd, m[0][r]));
    if (MAPS == 2) {
      // the difference replaces map 1's sums; columns past vd hold zeros
      const float f2 = lam / (lsum[MAPS - 1][r] + wa_sink(vw, hd, m[MAPS - 1][r]));
      float ss = 0.f;
      #pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const float o = acc[0][nt][r] * f - acc[MAPS - 1][nt][r] * f2;
        acc[0][nt][r] = o;
        ss += o * o;
      }
      f = (1.0f - df.diff) / sqrtf(sm_row16_sum(ss) / (float)vd + df.eps);
    }
    if (qi >= nq) continue;
    bf16_t* dst = out + ((int64_t)(t0 + qi) * H + hd) * vd;
    const bf16_t* gp = (gate != nullptr) ? gate + (int64_t)(t0 + qi) * ldg + hd * gs : nullptr;
    if (gp != nullptr && gs == 1) f *= sm_sigmoid(__bfloat162float(gp[0]));
    #pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const int col = nt * 16 + lrow;
      if (col < vd) {
        float o = acc[0][nt][r] * f;
        if (gp != nullptr && gs > 1) o *= sm_sigmoid(__bfloat162float(gp[col]));
        dst[col] = __float2bfloat16(o);
      }
    }
  }
}

#define WAM_KEYS 32   // keys per block

size_t wam_lds_bytes(int KD, int vd, bool dist, int maps) {
  const int ksteps = (KD + 31) / 32, KP = maps * ksteps * 32 + 8, NVp = (vd + 15) / 16 * 16;
  const int KB = WAM_KEYS;
  return (size_t)KB * KP * 2 + (size_t)NVp * (KB + 8) * 2 + 4 * 16 * (KB + 4) * 4 + KB * 4 +
         (dist ? 4 * (KB + 16) * 4 : 0);
}

}  // namespace

// 16-byte pieces of the cache rows: the key columns a head meets (dim, or
// kv_heads * dim for folded queries) and the value size are multiples of 8
bool window_attention_mfma_fits(int KD, int vd, int maps, bool dist, bool ext) {
  return !(ext && (dist || maps == 2)) && KD % 8 == 0 && vd % 8 == 0 &&
         KD <= (maps == 2 ? 128 : 512) && vd <= 256 &&
         wam_lds_bytes(KD, vd, true, maps) <= 150 * 1024;
}

void window_attention_mfma(torch::Tensor q, int KD, torch::Tensor cache, int H, int G, int dk, int vd,
                           int whole_key, torch::Tensor block_tables, int block_size,
                           torch::Tensor positions, float scale, wa_view vw,
                           const float* r1, const float* r2, const void* gate, int64_t ldg, int gs,
                           int maps, wa_diff df, torch::Tensor tiles, torch::Tensor out) {
  const int ntiles = tiles.size(0);
  if (q.size(0) == 0 || ntiles == 0) return;
  auto stream = at::cuda::getCurrentCUDAStream();
  const size_t lds = wam_lds_bytes(KD, vd, r1 != nullptr, maps);
  dim3 grid(ntiles, H);
#define WAM_LAUNCH(NT, KS, DIST, MAPS, EXT)                                                    \
  do {                                                                                         \
    auto kern = window_attention_mfma_kernel<NT, KS, WAM_KEYS, DIST, MAPS, EXT>;                  \
    static int raised = 0;                                                                     \
    if (lds > 64 * 1024 && (int)lds > raised) {                                                \
      TORCH_CHECK(hipFuncSetAttribute(reinterpret_cast<const void*>(kern),                     \
                      hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess,     \
                  "window attention: cannot raise the LDS limit");                             \
      raised = (int)lds;                                                                       \
    }                                                                                          \
    kern<<<grid, 256, lds, stream>>>(                                                          \
        reinterpret_cast<const bf16_t*>(q.data_ptr()), KD,                                     \
        reinterpret_cast<const bf16_t*>(cache.data_ptr()), block_tables.data_ptr<int>(),       \
        (int)block_tables.size(1), block_size, positions.data_ptr<int>(), tiles.data_ptr<int>(), \
        H, G, dk, vd, whole_key, scale, vw, r1, r2,                                            \
        reinterpret_cast<const bf16_t*>(gate), ldg, gs, df,                                    \
        reinterpret_cast<bf16_t*>(out.data_ptr()));                                            \
  } while (0)
#define WAM_BY_KS(NT, DIST, EXT)                             \
  do {                                                       \
    if (KD <= 128) WAM_LAUNCH(NT, 4, DIST, 1, EXT);          \
    else if (KD <= 256) WAM_LAUNCH(NT, 8, DIST, 1, EXT);     \
    else WAM_LAUNCH(NT, 16, DIST, 1, EXT);                   \
  } while (0)
#define WAM_BY_KS2(NT)                                       \
  do {                                                       \
    if (KD <= 64) WAM_LAUNCH(NT, 2, false, 2, false);        \
    else WAM_LAUNCH(NT, 4, false, 2, false);                 \
  } while (0)
#define WAM_BY_NT(BY, ...)                                   \
  do {                                                       \
    if (vd <= 64) BY(4, ##__VA_ARGS__);                      \
    else if (vd <= 128) BY(8, ##__VA_ARGS__);                \
    else BY(16, ##__VA_ARGS__);                              \
  } while (0)
  // chunks and capped scores: one map without distance bias (the caller sends
  // the rest of the combinations to the other kernels)
  if (maps == 2) WAM_BY_NT(WAM_BY_KS2);
  else if (r1 != nullptr) WAM_BY_NT(WAM_BY_KS, true, false);
  else if (vw.cap > 0.f || vw.chunk > 0) WAM_BY_NT(WAM_BY_KS, false, true);
  else WAM_BY_NT(WAM_BY_KS, false, false);
#undef WAM_BY_NT
#undef WAM_BY_KS2
#undef WAM_BY_KS
#undef WAM_LAUNCH
  SM_CHECK_LAUNCH();
}
