// Routed experts: fp32 router logits + sigmoid top-k, the expert-sorted row order of a
// prefill, and the weight-streaming expert GEMM of a decode step. The compute-bound prefill
// GEMMs run on gemm_tile.hip's persistent kernel with a per-tile expert (moe_gemm_tile).
#include "common.h"
#include "kernels.h"

namespace oamd {

namespace {

typedef __bf16 bf16x8m __attribute__((ext_vector_type(8)));

__device__ __forceinline__ f32x4 mfma16(u16x8 a, u16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8m, a), __builtin_bit_cast(bf16x8m, b), c, 0, 0, 0);
}

constexpr int kMaxExperts = 512;

// One wave: the `top` largest of z[0..E) (ties to the smaller index), their sigmoid scores and
// the ids, always inside [0, E). A NaN logit (a padding row's) counts as the smallest.
// NE: E <= 64 NE.
template <int NE>
__device__ __forceinline__ void wave_topk(const float* z, int E, int top, int lane, int* ids, float* weights) {
  float v[NE];
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    const float x = e < E ? z[e] : -INFINITY;
    v[i] = x == x ? x : -INFINITY;
  }
  unsigned taken = 0;   // bit i: expert lane + 64 i is chosen
  for (int k = 0; k < top; ++k) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = lane + 64 * i;
      if (e < E && !(taken >> i & 1) && (bi == 0x7fffffff || v[i] > best)) best = v[i], bi = e;
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(best, o, kWave);
      const int oi = __shfl_xor(bi, o, kWave);
      if (oi != 0x7fffffff && (bi == 0x7fffffff || ov > best || (ov == best && oi < bi))) best = ov, bi = oi;
    }
    if ((bi & 63) == lane) taken |= 1u << (bi >> 6);
    if (lane == 0) {
      ids[k] = bi;
      weights[k] = 1.f / (1.f + expf(-z[bi]));
    }
  }
}

}  // namespace

// 16 tokens per workgroup, 8 waves split K; experts in groups of NT MFMA tiles of 16, the waves'
// partial tiles summed through LDS into z[token][expert]. wr: [rows_w][K] rows (rows_w % (16 NT)
// == 0, rows past the last used one zero). NE: experts per lane of the top-k.
constexpr int kRouteWaves = 8;

template <int NT, int NE>
__global__ void __launch_bounds__(kRouteWaves * 64) moe_route_kernel(const bf16_t* __restrict__ h, const bf16_t* __restrict__ wr,
                                                        int T, int K, int E, int rows_w, int top, int* __restrict__ ids,
                                                        float* __restrict__ weights, float* __restrict__ gate,
                                                        float* __restrict__ logits) {
  constexpr int U = NT == 1 ? 16 : NT == 2 ? 8 : 4;   // K steps whose loads are in flight together
  extern __shared__ __attribute__((aligned(16))) float sm[];
  float* red = sm;                              // [waves][NT][256]
  float* z = sm + kRouteWaves * NT * 256;       // [16][rows_w]
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int l15 = lane & 15, lq = lane >> 4;
  const int t0 = blockIdx.x * 16;
  const bf16_t* hp = h + (int64_t)min(t0 + l15, T - 1) * K + 8 * lq;
  const int steps = K / 32;
  for (int e0 = 0; e0 < rows_w; e0 += 16 * NT) {
    f32x4 acc[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    const bf16_t* wp = wr + (int64_t)(e0 + l15) * K + 8 * lq;
    int s = w;
    for (; s + (U - 1) * kRouteWaves < steps; s += U * kRouteWaves) {
      u16x8 b[U], wv[U][NT];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = 32 * (s + u * kRouteWaves);
        b[u] = *reinterpret_cast<const u16x8*>(hp + k);
#pragma unroll
        for (int i = 0; i < NT; ++i) wv[u][i] = *reinterpret_cast<const u16x8*>(wp + (int64_t)16 * i * K + k);
      }
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int i = 0; i < NT; ++i) acc[i] = mfma16(wv[u][i], b[u], acc[i]);
    }
    for (; s < steps; s += kRouteWaves) {
      const u16x8 b = *reinterpret_cast<const u16x8*>(hp + 32 * s);
#pragma unroll
      for (int i = 0; i < NT; ++i)
        acc[i] = mfma16(*reinterpret_cast<const u16x8*>(wp + (int64_t)16 * i * K + 32 * s), b, acc[i]);
    }
    __syncthreads();   // red of the previous expert group is consumed
#pragma unroll
    for (int i = 0; i < NT; ++i) *reinterpret_cast<f32x4*>(red + ((w * NT + i) * 64 + lane) * 4) = acc[i];
    __syncthreads();
    for (int x = tid; x < NT * 256; x += kRouteWaves * 64) {   // tile i, lane l, register j: expert 16 i + 4 (l >> 4) + j, token l & 15
      const int i = x >> 8, l = (x >> 2) & 63, j = x & 3;
      float v = 0.f;
#pragma unroll
      for (int ww = 0; ww < kRouteWaves; ++ww) v += red[((ww * NT + i) * 64 + l) * 4 + j];
      z[(l & 15) * rows_w + e0 + 16 * i + 4 * (l >> 4) + j] = v;
    }
  }
  __syncthreads();
  for (int i = w; i < 16; i += kRouteWaves) {
    const int t = t0 + i;
    if (t >= T) break;
    wave_topk<NE>(z + i * rows_w, E, top, lane, ids + (int64_t)t * top, weights + (int64_t)t * top);
    if (gate && lane == 0) gate[t] = z[i * rows_w + E];
    if (logits)
      for (int e = lane; e < E; e += 64) logits[(int64_t)t * E + e] = z[i * rows_w + e];
  }
}

int moe_route(const bf16_t* h, const bf16_t* wr, int T, int K, int E, int rows_w, int top, int* ids, float* weights,
              float* gate, float* logits, hipStream_t stream) {
  if (T == 0) return 0;
  if (K % 32 || rows_w % 16 || E + (gate ? 1 : 0) > rows_w || E < 1 || E > kMaxExperts || top < 1 || top > E) return -1;
  const int NT = rows_w % 64 == 0 ? 4 : rows_w % 32 == 0 ? 2 : 1;
  const size_t lds = (kRouteWaves * NT * 256 + 16 * (size_t)rows_w) * sizeof(float);
  if (lds > 128 * 1024) return -2;
  const int grid = (T + 15) / 16, nt = kRouteWaves * 64;
#define OAMD_ROUTE(NTT, NEE) \
  moe_route_kernel<NTT, NEE><<<grid, nt, lds, stream>>>(h, wr, T, K, E, rows_w, top, ids, weights, gate, logits)
#define OAMD_ROUTE_E(NTT)                                             \
  if (E <= 64) OAMD_ROUTE(NTT, 1);                                    \
  else if (E <= 128) OAMD_ROUTE(NTT, 2);                              \
  else OAMD_ROUTE(NTT, kMaxExperts / 64)
  if (NT == 1) {
    OAMD_ROUTE_E(1);
  } else if (NT == 2) {
    OAMD_ROUTE_E(2);
  } else {
    OAMD_ROUTE_E(4);
  }
#undef OAMD_ROUTE_E
#undef OAMD_ROUTE
  OAMD_LAUNCH_CHECK();
  return 0;
}

// Top-k over finished fp32 logits [T][ld] (column E: the gate row).
__global__ void __launch_bounds__(256) moe_topk_kernel(const float* __restrict__ logits, int ld, int T, int E, int top,
                                                       int* __restrict__ ids, float* __restrict__ weights,
                                                       float* __restrict__ gate) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= T) return;
  const float* z = logits + (int64_t)t * ld;
  wave_topk<kMaxExperts / 64>(z, E, top, lane, ids + (int64_t)t * top, weights + (int64_t)t * top);
  if (gate && lane == 0) gate[t] = z[E];
}

int moe_topk(const float* logits, int ld, int T, int E, int top, int* ids, float* weights, float* gate,
             hipStream_t stream) {
  if (T == 0) return 0;
  if (E < 1 || E > kMaxExperts || top < 1 || top > E || ld < E + (gate ? 1 : 0)) return -1;
  moe_topk_kernel<<<(T + 3) / 4, 256, 0, stream>>>(logits, ld, T, E, top, ids, weights, gate);
  OAMD_LAUNCH_CHECK();
  return 0;
}

// One workgroup: histogram, padded offsets, then a row per slot (the order inside a segment is
// arbitrary: rows are independent).
__global__ void __launch_bounds__(1024) moe_sort_kernel(const int* __restrict__ ids, const float* __restrict__ weights,
                                                        int slots, int top, int E, int bm, int max_rows,
                                                        int* __restrict__ pos, int* __restrict__ src,
                                                        float* __restrict__ rscale, int* __restrict__ gtab) {
  __shared__ int cnt[kMaxExperts], off[kMaxExperts + 1], cur[kMaxExperts];
  const int tid = threadIdx.x;
  for (int e = tid; e < E; e += 1024) cnt[e] = cur[e] = 0;
  __syncthreads();
  for (int i = tid; i < slots; i += 1024) atomicAdd(&cnt[ids[i]], 1);
  __syncthreads();
  for (int e = tid; e <= E; e += 1024) {
    int o = 0;
    for (int f = 0; f < e; ++f) o += (cnt[f] + bm - 1) / bm * bm;
    off[e] = o;
  }
  __syncthreads();
  const int total = min(off[E], max_rows);
  for (int p = tid; p < total; p += 1024) {
    src[p] = -1;
    rscale[p] = 0.f;
  }
  for (int e = tid; e < E; e += 1024)
    for (int p = off[e]; p < off[e + 1]; p += bm) gtab[1 + p / bm] = e;
  if (tid == 0) gtab[0] = total / bm;
  __syncthreads();   // (global src / rscale: same workgroup, ordered by the barrier's fence)
  for (int i = tid; i < slots; i += 1024) {
    const int e = ids[i];
    const int p = off[e] + atomicAdd(&cur[e], 1);
    pos[i] = p;
    src[p] = i / top;
    rscale[p] = weights[i];
  }
}

int moe_sort(const int* ids, const float* weights, int slots, int top, int E, int bm, int max_rows, int* pos, int* src,
             float* rscale, int* gtab, hipStream_t stream) {
  if (slots == 0) return 0;
  if (E < 1 || E > kMaxExperts || bm < 1 || top < 1 || max_rows % bm) return -1;
  // every assignment fits: at most slots rows plus bm - 1 padding rows per non-empty expert
  if ((int64_t)max_rows < (int64_t)slots + (int64_t)(E < slots ? E : slots) * (bm - 1)) return -2;
  moe_sort_kernel<<<1, 1024, 0, stream>>>(ids, weights, slots, top, E, bm, max_rows, pos, src, rscale, gtab);
  OAMD_LAUNCH_CHECK();
  return 0;
}

__global__ void __launch_bounds__(256) moe_gather_kernel(const uint4* __restrict__ h, const int* __restrict__ src,
                                                         const int* __restrict__ gtab, int bm, uint4* __restrict__ xp,
                                                         int vecs) {
  const int p = blockIdx.x;
  if (p >= gtab[0] * bm) return;
  const int t = src[p];
  for (int i = threadIdx.x; i < vecs; i += 256)
    xp[(int64_t)p * vecs + i] = t >= 0 ? h[(int64_t)t * vecs + i] : make_uint4(0, 0, 0, 0);
}

int moe_gather(const void* h, const int* src, const int* gtab, int bm, int max_rows, void* xp, int row_bytes,
               hipStream_t stream) {
  if (max_rows == 0) return 0;
  if (row_bytes % 16) return -1;
  moe_gather_kernel<<<max_rows, 256, 0, stream>>>(static_cast<const uint4*>(h), src, gtab, bm, static_cast<uint4*>(xp),
                                                  row_bytes / 16);
  OAMD_LAUNCH_CHECK();
  return 0;
}

// Expert GEMM for few rows per expert: the structure of gemm_skinny.hip (W straight to VGPRs as
// the MFMA A fragment, 4 waves split K, partial tiles summed through LDS) with the expert in
// blockIdx.y. A workgroup lists the slots routed to its expert, then walks them 16 * MT at a
// time; an expert nobody chose costs one read of the id list. NT = 2: the SwiGLU pair (16 gate
// rows and the 16 matching up rows of the 64-row interleave).
constexpr int kMaxSlots = 4096;

template <int NT, int MT>
__global__ void __launch_bounds__(256) moe_skinny_kernel(const bf16_t* __restrict__ X, const bf16_t* __restrict__ W,
                                                         bf16_t* __restrict__ Y, const int* __restrict__ ids,
                                                         const float* __restrict__ weights, int slots, int div, int N,
                                                         int K) {
  constexpr int U = 8;
  __shared__ float red[4][NT * MT][256];
  __shared__ unsigned short list[kMaxSlots];
  __shared__ int count;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int r = lane & 15, kq = lane >> 4;
  const int ex = blockIdx.y;
  if (tid == 0) count = 0;
  __syncthreads();
  for (int i = tid; i < slots; i += 256)
    if (ids[i] == ex) list[atomicAdd(&count, 1)] = (unsigned short)i;
  __syncthreads();
  const int n = count;
  if (n == 0) return;

  int rows[NT];
  if constexpr (NT == 2) {
    const int g = blockIdx.x >> 2, sub = blockIdx.x & 3;
    rows[0] = g * 128 + sub * 16;
    rows[1] = g * 128 + 64 + sub * 16;
  } else {
    rows[0] = blockIdx.x * 16;
  }
  const int steps = K / 32;
  const int s0 = steps * w / 4, s1 = steps * (w + 1) / 4;
  const u16x8* wp[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
    wp[t] = reinterpret_cast<const u16x8*>(W + ((int64_t)ex * N + rows[t] + r) * K + kq * 8);
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};

  for (int c0 = 0; c0 < n; c0 += 16 * MT) {
    const u16x8* xp[MT];
    bool xv[MT];
#pragma unroll
    for (int j = 0; j < MT; ++j) {
      const int m = c0 + j * 16 + r;
      xv[j] = m < n;
      xp[j] = reinterpret_cast<const u16x8*>(X + (int64_t)(list[xv[j] ? m : 0] / div) * K + kq * 8);
    }
    f32x4 acc[NT][MT];
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int j = 0; j < MT; ++j) acc[t][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    int s = s0;
    for (; s + U <= s1; s += U) {
      u16x8 a[U][NT], b[U][MT];
#pragma unroll
      for (int u = 0; u < U; ++u) {
#pragma unroll
        for (int t = 0; t < NT; ++t) a[u][t] = wp[t][(s + u) * 4];
#pragma unroll
        for (int j = 0; j < MT; ++j) b[u][j] = xv[j] ? xp[j][(s + u) * 4] : zero;
      }
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
          for (int j = 0; j < MT; ++j) acc[t][j] = mfma16(a[u][t], b[u][j], acc[t][j]);
    }
    for (; s < s1; ++s) {
      u16x8 a[NT], b[MT];
#pragma unroll
      for (int t = 0; t < NT; ++t) a[t] = wp[t][s * 4];
#pragma unroll
      for (int j = 0; j < MT; ++j) b[j] = xv[j] ? xp[j][s * 4] : zero;
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int j = 0; j < MT; ++j) acc[t][j] = mfma16(a[t], b[j], acc[t][j]);
    }
    __syncthreads();   // the previous round's sums are consumed
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int j = 0; j < MT; ++j)
        *reinterpret_cast<f32x4*>(&red[w][t * MT + j][lane * 4]) = acc[t][j];
    __syncthreads();
    // lane l, register i of a tile: W row 4 (l >> 4) + i, X row l & 15; 4 rows per thread
    for (int x = tid; x < MT * 64; x += 256) {
      const int j = x >> 6, l = x & 63;
      const int m = c0 + j * 16 + (l & 15);
      if (m >= n) continue;
      f32x4 v[NT];
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        v[t] = *reinterpret_cast<const f32x4*>(&red[0][t * MT + j][l * 4]);
#pragma unroll
        for (int ww = 1; ww < 4; ++ww) v[t] += *reinterpret_cast<const f32x4*>(&red[ww][t * MT + j][l * 4]);
      }
      const int slot = list[m];
      f32x4 o = v[0];
      int64_t at;
      if constexpr (NT == 2) {
        const float c = weights[slot];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float g = c * v[0][i], u = c * v[1][i];
          o[i] = g / (1.f + __expf(-g)) * u;
        }
        at = (int64_t)slot * (N / 2) + (blockIdx.x >> 2) * 64 + (blockIdx.x & 3) * 16 + 4 * (l >> 4);
      } else {
        at = (int64_t)slot * N + rows[0] + 4 * (l >> 4);
      }
      *reinterpret_cast<uint2*>(Y + at) = make_uint2(pack_bf2(o[0], o[1]), pack_bf2(o[2], o[3]));
    }
  }
}

int moe_gemm_skinny(const bf16_t* X, const bf16_t* W, bf16_t* Y, const int* ids, const float* weights, int slots,
                    int div, int E, int N, int K, bool silu_gu, hipStream_t stream) {
  if (slots == 0) return 0;
  if (slots > kMaxSlots || K % 32 || div < 1) return -1;
  if (silu_gu ? N % 128 : N % 16) return -2;
  const dim3 grid(silu_gu ? N / 32 : N / 16, E);
  const int mt = slots <= 8 * (int64_t)E ? 1 : slots <= 20 * (int64_t)E ? 2 : 4;   // by the rows an expert gets on average
  if (silu_gu) {
    if (mt == 1) moe_skinny_kernel<2, 1><<<grid, 256, 0, stream>>>(X, W, Y, ids, weights, slots, div, N, K);
    else if (mt == 2) moe_skinny_kernel<2, 2><<<grid, 256, 0, stream>>>(X, W, Y, ids, weights, slots, div, N, K);
    else moe_skinny_kernel<2, 4><<<grid, 256, 0, stream>>>(X, W, Y, ids, weights, slots, div, N, K);
  } else {
    if (mt == 1) moe_skinny_kernel<1, 1><<<grid, 256, 0, stream>>>(X, W, Y, ids, weights, slots, div, N, K);
    else if (mt == 2) moe_skinny_kernel<1, 2><<<grid, 256, 0, stream>>>(X, W, Y, ids, weights, slots, div, N, K);
    else moe_skinny_kernel<1, 4><<<grid, 256, 0, stream>>>(X, W, Y, ids, weights, slots, div, N, K);
  }
  OAMD_LAUNCH_CHECK();
  return 0;
}

}  // namespace oamd
