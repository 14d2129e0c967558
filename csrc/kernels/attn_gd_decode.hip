// Paged decode attention with any query/key size and any value size (each up to 256), GQA,
// split over the context: both products on MFMA.
//
// Workgroup = (sequence, split, key/value head, chunk of up to 16 query heads); 4 waves, each
// walking its own 32-token chunks (two 16-token cache tiles) with the next chunk's K and V
// registers in flight. The cache tiles (qkv_heads.hip) are laid out as MFMA fragments, so
// every load is one contiguous 1 KiB wave access:
//   S = K Q^T     v_mfma_f32_16x16x32_bf16, A = K tile (token rows), B = q (one head per
//                 column): lane (head l & 15, group l >> 4) ends with tokens 4 (l >> 4) + i
//   O^T += V^T P  v_mfma_f32_16x16x16_bf16, A = V^T tile, B = P, which is exactly the layout
//                 S left in the registers; a lane's column is one head, so the softmax
//                 rescale is lane-local
// The waves are merged through LDS; sequences cut into several splits leave fp32 partials
// for the combine kernel. With a window only the last `window` tokens are read.
#include "attn_gd.h"

namespace oamd {

using namespace gd;

namespace {

constexpr int kTok = 32;            // tokens per wave chunk
constexpr int kChunk = 4 * kTok;    // tokens per workgroup round
constexpr int kMaxPages = 1024;     // page ids of one split staged in LDS

// tokens of one split of `len`, a multiple of `round`
__device__ __forceinline__ int split_tokens(int len, int num_splits, int round) {
  const int per = (len + num_splits - 1) / num_splits;
  return (per + round - 1) / round * round;
}

// first token a windowed query reads, down to a whole cache tile
__device__ __forceinline__ int window_start(int len, int window) { return max(0, len - window) & ~15; }

template <int NK, int NV>
struct Frag {
  u16x8 k[2][NK];   // [tile][32-dim step]
  u16x8 v[2][NV];   // [tile][32-dim block]: low half dims 0-15, high half 16-31, 4 tokens each
};

}  // namespace

// NK, NV: 32-dim steps of the instantiated key / value sizes
template <int NK, int NV>
__global__ void __launch_bounds__(256, (NK + NV <= 8) ? 2 : 1) attn_gd_decode_kernel(const AttnDecode a) {
  constexpr int DV = 32 * NV;
  __shared__ int pg[kMaxPages];
  __shared__ __attribute__((aligned(16))) float red[4][16][DV];
  __shared__ float mls[4][16][2];
  const int hcs = (a.G + 15) / 16;   // head chunks
  const int vh = blockIdx.x % (a.Hkv * hcs);
  const int rest = blockIdx.x / (a.Hkv * hcs);
  const int b = rest / a.num_splits, s = rest % a.num_splits;
  const int kvh = vh / hcs, h0 = (vh % hcs) * 16;
  const int nh = min(16, a.G - h0);
  const int Hq = a.Hkv * a.G;
  const int len = min(a.seq_lens[b], a.max_pages * a.page_size);
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, lg = lane >> 4;
  bf16_t* orow = a.out + (int64_t)b * a.o_ld + (kvh * a.G + h0) * a.dvp;
  if (len <= 0) {   // padding row: zeros, written once
    if (s == 0)
      for (int e = tid; e < nh * a.dvp; e += 256) orow[e] = 0;
    return;
  }
  const int first = window_start(len, a.window);   // tokens below len - window share its tile and are masked
  const int per = split_tokens(len - first, a.num_splits, kChunk);
  const int start = first + s * per;
  if (start >= len) return;
  const int end = min(len, start + per);
  const int ns_b = (len - first + per - 1) / per;
  const int lo = len - a.window;
  const int nch = (end - start + kTok - 1) / kTok;

  const int page0 = start >> a.log2_page;
  const int npg = ((end - 1) >> a.log2_page) - page0 + 1;
  const int* btb = a.block_tables + (int64_t)b * a.max_pages + page0;
  for (int i = tid; i < npg; i += 256) pg[i] = btb[i];

  u16x8 qf[NK];
#pragma unroll
  for (int st = 0; st < NK; ++st) {
    const int d = 32 * st + 8 * lg;
    qf[st] = (l15 < nh && d < a.dkp)
                 ? *reinterpret_cast<const u16x8*>(a.q + ((int64_t)b * Hq + kvh * a.G + h0 + l15) * a.dkp + d)
                 : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
  }
  __syncthreads();

  const int last_tile = (end - 1) & ~15;
  const int nkc = (a.dkp >> 3) - 1, nvb = (a.dvp >> 5) - 1;
  auto load = [&](Frag<NK, NV>& r, int c) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int t0 = min(start + c * kTok + 16 * i, last_tile);   // past the end: the last tile again, masked
      const int64_t head = ((int64_t)pg[(t0 >> a.log2_page) - page0] * a.Hkv + kvh) * a.page_size + (t0 & (a.page_size - 1));
      const bf16_t* kp = a.k_cache + head * a.dkp + l15 * 8;
      const bf16_t* vp = a.v_cache + head * a.dvp + (lg * 16 + l15) * 8;
#pragma unroll
      for (int st = 0; st < NK; ++st)   // dims past dkp: any finite chunk, q is zero there
        r.k[i][st] = __builtin_nontemporal_load(reinterpret_cast<const u16x8*>(kp + min(4 * st + lg, nkc) * 128));
#pragma unroll
      for (int m = 0; m < NV; ++m)      // dims past dvp: computed, never stored
        r.v[i][m] = __builtin_nontemporal_load(reinterpret_cast<const u16x8*>(vp + min(m, nvb) * 512));
    }
  };

  float m_run = -1e30f, l_run = 0.f;   // finite start: no inf - inf
  f32x4 acc[2 * NV];
#pragma unroll
  for (int m = 0; m < 2 * NV; ++m) acc[m] = f32x4{0.f, 0.f, 0.f, 0.f};

  auto consume = [&](Frag<NK, NV>& r, int c) {
    const int base = start + c * kTok;
    float sc[2][4];
    float mx = m_run;
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      f32x4 d = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int st = 0; st < NK; ++st) d = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf8(r.k[i][st]), bf8(qf[st]), d, 0, 0, 0);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int t = base + 16 * i + 4 * lg + j;
        sc[i][j] = t < end && t >= lo ? d[j] * a.scale_log2 : -INFINITY;
        mx = fmaxf(mx, sc[i][j]);
      }
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
    mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
    if (__any(mx > m_run)) {
      const float alpha = exp2f(m_run - mx);
      l_run *= alpha;
#pragma unroll
      for (int m = 0; m < 2 * NV; ++m) acc[m] *= alpha;
      m_run = mx;
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      f32x4 p;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        p[j] = exp2f(sc[i][j] - m_run);
        l_run += p[j];
      }
      const s16x4 pb = __builtin_bit_cast(s16x4, __builtin_convertvector(p, bf16x4));
      const int left = end - (base + 16 * i + 4 * lg);   // this lane's 4 tokens that exist
#pragma unroll
      for (int m = 0; m < NV; ++m) {
        u16x8 v = r.v[i][m];
        if (left < 4) {   // stale cache rows past the end must not reach the product, not even times 0
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (j >= left) v[j] = v[4 + j] = 0;
        }
        const s16x8 vs = __builtin_bit_cast(s16x8, v);
        acc[2 * m] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_shufflevector(vs, vs, 0, 1, 2, 3), pb, acc[2 * m], 0, 0, 0);
        acc[2 * m + 1] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_shufflevector(vs, vs, 4, 5, 6, 7), pb, acc[2 * m + 1], 0, 0, 0);
      }
    }
  };

  {
    Frag<NK, NV> ra, rb;
    if (w < nch) load(ra, w);
    for (int c = w; c < nch; c += 8) {
      if (c + 4 < nch) load(rb, c + 4);
      consume(ra, c);
      if (c + 4 < nch) {
        if (c + 8 < nch) load(ra, c + 8);
        consume(rb, c + 4);
      }
    }
  }
  l_run += __shfl_xor(l_run, 16, kWave);
  l_run += __shfl_xor(l_run, 32, kWave);
  if (l15 < nh) {
#pragma unroll
    for (int m = 0; m < 2 * NV; ++m) *reinterpret_cast<f32x4*>(&red[w][l15][16 * m + 4 * lg]) = acc[m];
    if (lg == 0) {
      mls[w][l15][0] = m_run;
      mls[w][l15][1] = l_run;
    }
  }
  __syncthreads();
  for (int e = tid; e < nh * a.dvp; e += 256) {
    const int h = e / a.dvp, d = e % a.dvp;
    float M = mls[0][h][0];
#pragma unroll
    for (int ww = 1; ww < 4; ++ww) M = fmaxf(M, mls[ww][h][0]);
    float o = 0.f, L = 0.f;
#pragma unroll
    for (int ww = 0; ww < 4; ++ww) {
      const float f = exp2f(mls[ww][h][0] - M);
      o += f * red[ww][h][d];
      L += f * mls[ww][h][1];
    }
    if (ns_b == 1) {
      if (a.gate) o *= a.gate[(int64_t)b * Hq + kvh * a.G + h0 + h];
      orow[e] = f2bf(L > 0.f ? o / L : 0.f);
    } else {
      const int64_t bh = (int64_t)b * Hq + kvh * a.G + h0 + h;
      a.o_part[(bh * a.num_splits + s) * a.dvp + d] = o;
      if (d == 0) {
        a.ml_part[(bh * a.num_splits + s) * 2] = M;
        a.ml_part[(bh * a.num_splits + s) * 2 + 1] = L;
      }
    }
  }
}

// Sum the partials of sequences cut into several splits: grid (B, Hq).
__global__ void __launch_bounds__(256) attn_gd_combine_kernel(const AttnDecode a, int round) {
  const int b = blockIdx.x, hq = blockIdx.y, Hq = gridDim.y;
  const int len = min(a.seq_lens[b], a.max_pages * a.page_size);
  if (len <= 0) return;
  const int n = len - window_start(len, a.window);
  const int per = split_tokens(n, a.num_splits, round);
  const int ns = (n + per - 1) / per;
  if (ns == 1) return;
  const int64_t bh = (int64_t)b * Hq + hq;
  const float* ml = a.ml_part + bh * a.num_splits * 2;
  float M = -INFINITY;
  for (int s = 0; s < ns; ++s) M = fmaxf(M, ml[2 * s]);
  float L = 0.f;
  for (int s = 0; s < ns; ++s) L += exp2f(ml[2 * s] - M) * ml[2 * s + 1];
  float inv = L > 0.f ? 1.f / L : 0.f;
  if (a.gate) inv *= a.gate[bh];
  for (int d = threadIdx.x; d < a.dvp; d += blockDim.x) {
    float o = 0.f;
    for (int s = 0; s < ns; ++s) o += exp2f(ml[2 * s] - M) * a.o_part[(bh * a.num_splits + s) * a.dvp + d];
    a.out[b * (int64_t)a.o_ld + hq * a.dvp + d] = f2bf(o * inv);
  }
}

template <int NK>
static int launch_nv(const AttnDecode& a, int grid, hipStream_t stream) {
  switch (dim_bin(a.dvp)) {
    case 32: attn_gd_decode_kernel<NK, 1><<<grid, 256, 0, stream>>>(a); break;
    case 64: attn_gd_decode_kernel<NK, 2><<<grid, 256, 0, stream>>>(a); break;
    case 96: attn_gd_decode_kernel<NK, 3><<<grid, 256, 0, stream>>>(a); break;
    case 128: attn_gd_decode_kernel<NK, 4><<<grid, 256, 0, stream>>>(a); break;
    case 192:
    case 256: attn_gd_decode_kernel<NK, 8><<<grid, 256, 0, stream>>>(a); break;
    default: return -2;
  }
  return 0;
}

int attn_gd_decode(const AttnDecode& a, int B, hipStream_t stream) {
  if (B == 0) return 0;
  if (a.dkp % 8 || a.dvp % 32 || a.G < 1 || a.page_size % 16 || a.max_pages > kMaxPages || a.num_splits < 1 || a.window < 1) return -1;
  const int grid = B * a.num_splits * a.Hkv * ((a.G + 15) / 16);
  int rc = -2;
  switch (dim_bin(a.dkp)) {
    case 32: rc = launch_nv<1>(a, grid, stream); break;
    case 64: rc = launch_nv<2>(a, grid, stream); break;
    case 96: rc = launch_nv<3>(a, grid, stream); break;
    case 128: rc = launch_nv<4>(a, grid, stream); break;
    case 192: rc = launch_nv<6>(a, grid, stream); break;
    case 256: rc = launch_nv<8>(a, grid, stream); break;
    default: break;
  }
  if (rc != 0) return rc;
  OAMD_LAUNCH_CHECK();
  return a.num_splits > 1 ? attn_combine(a, B, kChunk, stream) : 0;
}

int attn_combine(const AttnDecode& a, int B, int round, hipStream_t stream) {
  attn_gd_combine_kernel<<<dim3(B, a.Hkv * a.G), a.dvp > 128 ? 256 : 64, 0, stream>>>(a, round);
  OAMD_LAUNCH_CHECK();
  return 0;
}

}  // namespace oamd
