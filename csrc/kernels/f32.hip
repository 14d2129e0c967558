// True 32-bit forms of the model's products, for models served in fp32 (no reduced-precision
// matrix mode anywhere): a tiled GEMM (plain, SwiGLU, per-expert row groups) and attention
// for any head size. Precision first: fp32 FMA on the vector units.
#include "common.h"
#include "kernels.h"

namespace oamd {

// Y[M, N] = X[M, K] W[N, K]^T, 64 x 64 tiles, 256 threads x 4 x 4 outputs.
// SILU: W holds gate | up rows interleaved in 64-row blocks; a tile is 64 features, Y [M, N/2]
// = silu(c g) * (c u) with c the row's scale (rscale, or 1).
// gtab != nullptr: rows are expert segments padded to 64-row tiles; gtab[0] = tile count,
// gtab[1 + i] = expert of tile i, W [experts][N][K].
template <bool SILU>
__global__ void __launch_bounds__(256) gemm_f32_kernel(const float* __restrict__ X, const float* __restrict__ W,
                                                       float* __restrict__ Y, int M, int N, int K, int ldy,
                                                       const int* __restrict__ gtab, const float* __restrict__ rscale,
                                                       GluAct act, int64_t ldx, int64_t xh, int64_t yh) {
  constexpr int NB = SILU ? 2 : 1;
  __shared__ float xs[16][64 + 4];
  __shared__ float ws[NB][16][64 + 4];
  const int m0 = blockIdx.x * 64, f0 = blockIdx.y * 64;
  if (gtab) {
    if ((int)blockIdx.x >= gtab[0]) return;
    W += (int64_t)gtab[1 + blockIdx.x] * N * K;
  }
  if (blockIdx.z) {   // one product per head
    X += blockIdx.z * xh;
    W += (int64_t)blockIdx.z * N * K;
    Y += blockIdx.z * yh;
  }
  const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  const int lr = tid >> 2, lk = (tid & 3) * 4;   // loader: row, 4 consecutive k
  float acc[NB][4][4] = {};
  for (int k0 = 0; k0 < K; k0 += 16) {
    __syncthreads();
    {
      f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f};
      if (m0 + lr < M) v = *reinterpret_cast<const f32x4*>(X + (int64_t)(m0 + lr) * ldx + k0 + lk);
#pragma unroll
      for (int j = 0; j < 4; ++j) xs[lk + j][lr] = v[j];
    }
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const int wr = (SILU ? 2 * f0 + 64 * b : f0) + lr;
      f32x4 v = f32x4{0.f, 0.f, 0.f, 0.f};
      if (wr < N) v = *reinterpret_cast<const f32x4*>(W + (int64_t)wr * K + k0 + lk);
#pragma unroll
      for (int j = 0; j < 4; ++j) ws[b][lk + j][lr] = v[j];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 16; ++k) {
      float xv[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) xv[i] = xs[k][ty * 4 + i];
#pragma unroll
      for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float wv = ws[b][k][tx * 4 + j];
#pragma unroll
          for (int i = 0; i < 4; ++i) acc[b][i][j] = __builtin_fmaf(xv[i], wv, acc[b][i][j]);
        }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int m = m0 + ty * 4 + i;
    if (m >= M) continue;
    const float c = rscale ? rscale[m] : 1.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = f0 + tx * 4 + j;
      if (n >= (SILU ? N / 2 : N)) continue;
      float y = acc[0][i][j];
      if constexpr (SILU) {
        const float g = c * y, u = c * acc[NB - 1][i][j];
        y = g / (1.f + expf(-g * __builtin_fmaf(act.c, g * g, act.a))) * u;
      }
      Y[(int64_t)m * ldy + n] = y;
    }
  }
}

int gemm_f32(const float* X, const float* W, float* Y, int M, int N, int K, int ldy, int glu, const int* gtab,
             const float* rscale, hipStream_t stream) {
  if (M == 0) return 0;
  if (K % 16 || (glu && N % 128)) return -1;
  const int nf = glu ? N / 2 : N;
  const dim3 grid((M + 63) / 64, (nf + 63) / 64);
  if (glu) gemm_f32_kernel<true><<<grid, 256, 0, stream>>>(X, W, Y, M, N, K, ldy, gtab, rscale, glu_act(glu), K, 0, 0);
  else gemm_f32_kernel<false><<<grid, 256, 0, stream>>>(X, W, Y, M, N, K, ldy, gtab, rscale, GluAct{}, K, 0, 0);
  OAMD_LAUNCH_CHECK();
  return 0;
}

int head_gemm_f32(const float* X, const float* W, float* Y, int M, int N, int K, int H, int64_t ldx, int64_t xh,
                  int64_t ldy, int64_t yh, hipStream_t stream) {
  if (M == 0) return 0;
  if (K % 16 || ldx % 4 || xh % 4 || H < 1 || H > 65535) return -1;
  const dim3 grid((M + 63) / 64, (N + 63) / 64, H);
  gemm_f32_kernel<false><<<grid, 256, 0, stream>>>(X, W, Y, M, N, K, (int)ldy, nullptr, nullptr, GluAct{}, ldx, xh, yh);
  OAMD_LAUNCH_CHECK();
  return 0;
}

// Attention of one query row and head per workgroup; each of the 4 waves takes every fourth
// 64-key block (a key per lane), then owns NE output dims lane, lane + 64, ...
// PAGED: row b's keys come from the paged cache (token rows); else from packed k / v rows of
// the sequence holding the row, after the shared-prefix rows.
template <bool PAGED, int NE>
__global__ void __launch_bounds__(256) attn_f32_kernel(const AttnF32 a) {
  __shared__ float qs[64 * NE];
  __shared__ float ps[4][64];
  __shared__ float red[4][64 * NE];
  __shared__ float mls[4][2];
  const int t = blockIdx.x, hq = blockIdx.y, kvh = hq / (gridDim.y / a.Hkv);
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  float* out = a.o + (int64_t)t * a.o_ld + hq * a.dvp;
  int n = 0, pl = 0;
  int64_t base = 0;
  if constexpr (PAGED) {
    n = min(a.seq_lens[t], a.max_pages * a.page_size);
    if (n <= 0) {
      for (int d = tid; d < a.dvp; d += 256) out[d] = 0.f;
      return;
    }
  } else {
    int s = 0;
    while (s < a.num_seqs && a.cu_seqlens[s + 1] <= t) ++s;
    if (s >= a.num_seqs) return;   // padding row of a graph-captured prefill
    base = a.cu_seqlens[s];
    pl = a.seq_pfx ? a.seq_pfx[s] : 0;
    n = pl + t - (int)base + 1;
  }
  for (int d = tid; d < a.dkp; d += 256) qs[d] = a.q[((int64_t)t * gridDim.y + hq) * a.dkp + d];
  __syncthreads();
  // row index (in units of one head's row) of key j
  auto key = [&](int j, const float*& kp, const float*& vp) {
    if constexpr (PAGED) {
      const int64_t r = ((int64_t)a.block_tables[(int64_t)t * a.max_pages + j / a.page_size] * a.Hkv + kvh) * a.page_size + j % a.page_size;
      kp = a.k + r * a.k_ld;
      vp = a.v + r * a.v_ld;
    } else {
      const int64_t r = j < pl ? j : base + j - pl;
      kp = (j < pl ? a.pk : a.k) + (r * a.Hkv + kvh) * a.dkp;
      vp = (j < pl ? a.pv : a.v) + (r * a.Hkv + kvh) * a.dvp;
    }
  };
  float m = -1e30f, l = 0.f;
  float acc[NE] = {};
  const int lo = max(0, n - a.window);   // first key in the window
  for (int j0 = lo + w * 64; j0 < n; j0 += 256) {
    const int j = j0 + lane;
    float s = -INFINITY;
    if (j < n) {
      const float *kp, *vp;
      key(j, kp, vp);
      float d0 = 0.f;
      for (int d = 0; d < a.dkp; d += 4) {
        const f32x4 kv = *reinterpret_cast<const f32x4*>(kp + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) d0 = __builtin_fmaf(qs[d + e], kv[e], d0);
      }
      s = d0 * a.scale;
    }
    const float mn = fmaxf(m, wave_max(s));
    const float alpha = expf(m - mn);
    const float p = expf(s - mn);
    m = mn;
    l = l * alpha + wave_sum(p);
    ps[w][lane] = p;
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
    for (int e = 0; e < NE; ++e) acc[e] *= alpha;
    const int cnt = min(64, n - j0);
    for (int i = 0; i < cnt; ++i) {
      const float *kp, *vp;
      key(j0 + i, kp, vp);
#pragma unroll
      for (int e = 0; e < NE; ++e)
        if (lane + 64 * e < a.dvp) acc[e] = __builtin_fmaf(ps[w][i], vp[lane + 64 * e], acc[e]);
    }
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
  }
#pragma unroll
  for (int e = 0; e < NE; ++e) red[w][lane + 64 * e] = acc[e];
  if (lane == 0) {
    mls[w][0] = m;
    mls[w][1] = l;
  }
  __syncthreads();
  const float M = fmaxf(fmaxf(mls[0][0], mls[1][0]), fmaxf(mls[2][0], mls[3][0]));
  for (int d = tid; d < a.dvp; d += 256) {
    float o = 0.f, L = 0.f;
#pragma unroll
    for (int ww = 0; ww < 4; ++ww) {
      const float f = expf(mls[ww][0] - M);
      o += f * red[ww][d];
      L += f * mls[ww][1];
    }
    out[d] = a.gate ? o / L * a.gate[(int64_t)t * gridDim.y + hq] : o / L;
  }
}

int attn_f32(const AttnF32& a, int rows, int Hq, bool paged, hipStream_t stream) {
  if (rows == 0) return 0;
  const int top = a.dkp > a.dvp ? a.dkp : a.dvp;
  if (a.dkp % 4 || top > (paged ? 640 : 256) || Hq % a.Hkv || a.window < 1) return -1;
  if (paged && top > 256) attn_f32_kernel<true, 10><<<dim3(rows, Hq), 256, 0, stream>>>(a);
  else if (paged) attn_f32_kernel<true, 4><<<dim3(rows, Hq), 256, 0, stream>>>(a);
  else attn_f32_kernel<false, 4><<<dim3(rows, Hq), 256, 0, stream>>>(a);
  OAMD_LAUNCH_CHECK();
  return 0;
}

}  // namespace oamd
