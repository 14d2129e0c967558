// Paged decode attention over latent rows: every query head of a sequence reads the same cached row
// [c (rp) | rotated part | 0 .. ck), its score is the product with the whole row and its value is c.
//
// Workgroup = (sequence, split, 16 HG query heads), 4 HG waves, 64-token tiles. A tile is loaded once,
// held in registers while the previous one is worked on, and stored to LDS, from which both
// products read:
//   S = K Q^T     v_mfma_f32_16x16x32_bf16, A = rows (tokens x dims), B = q (one head per column);
//                 wave w of a head group takes tokens 16 w .. 16 w + 15
//   O^T += V^T P  the same instruction, A = the same rows through the transposing LDS read, B = P, which
//                 the head group's waves exchange through LDS; a wave takes every fourth 16-dim block
//                 of all tokens, so nothing is merged at the end
// A lane's column is one head in both, so softmax state is lane-local. Rows are padded by 16 bytes in
// LDS, which spreads both access patterns over the banks. Head chunks of one (sequence, split) run
// on one XCD and share its L2. Split sequences leave fp32 partials for the combine kernel of
// attn_gd_decode.hip.
#include "attn_gd.h"

namespace oamd {

using namespace gd;

namespace {

constexpr int kMaxPages = 1024;   // page ids of one split staged in LDS
constexpr int kRound = 64;        // tokens of a workgroup round

__device__ __forceinline__ int latent_split(int len, int num_splits) {
  const int per = (len + num_splits - 1) / num_splits;
  return (per + kRound - 1) / kRound * kRound;
}

}  // namespace

// NK: 32-dim steps of a row (even), ck = 32 NK; HG: groups of 16 heads
template <int NK, int HG>
__global__ void __launch_bounds__(256 * HG, HG == 1 && NK < 16 ? 2 : 1) attn_latent_decode_kernel(const AttnDecode a, int rp, int B) {
  constexpr int CK = 32 * NK, RK = 2 * CK + 16, NC = CK / 8, NT = 256 * HG, NL = NK / HG, NB = NK / 2;
  __shared__ int pg[kMaxPages];
  __shared__ __attribute__((aligned(16))) char tile[kRound * RK];
  __shared__ __attribute__((aligned(16))) s16x4 ps[HG][4][64];
  __shared__ float stat[HG][4][16];
  const int hcs = (a.G + 16 * HG - 1) / (16 * HG);
  const int items = B * a.num_splits;
  const int jj = blockIdx.x >> 3;
  const int item = (jj / hcs) * 8 + (blockIdx.x & 7);
  if (item >= items) return;
  const int b = item / a.num_splits, s = item % a.num_splits;
  const int tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int hg = wv >> 2, w = wv & 3, l15 = lane & 15, lg = lane >> 4;
  const int hb = (jj % hcs) * 16 * HG;             // the workgroup's first head
  const int h = hb + 16 * hg + l15;                // this lane's
  const int len = min(a.seq_lens[b], a.max_pages * a.page_size);
  if (len <= 0) {   // padding row: zeros, written once
    if (s == 0)
      for (int e = tid; e < min(16 * HG, a.G - hb) * rp; e += NT) a.out[(int64_t)b * a.o_ld + hb * rp + e] = 0;
    return;
  }
  const int per = latent_split(len, a.num_splits);
  const int start = s * per;
  if (start >= len) return;
  const int end = min(len, start + per);
  const int ns_b = (len + per - 1) / per;
  const int ntile = (end - start + kRound - 1) / kRound;

  const int page0 = start >> a.log2_page;
  const int npg = ((end - 1) >> a.log2_page) - page0 + 1;
  const int* btb = a.block_tables + (int64_t)b * a.max_pages + page0;
  for (int i = tid; i < npg; i += NT) pg[i] = btb[i];

  u16x8 qf[NK];
#pragma unroll
  for (int st = 0; st < NK; ++st)
    qf[st] = h < a.G ? *reinterpret_cast<const u16x8*>(a.q + ((int64_t)b * a.G + h) * CK + 32 * st + 8 * lg)
                     : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
  __syncthreads();

  u16x8 kr[NL];
  auto load = [&](int ti) {
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int c = NT * i + tid, row = c / NC, ch = c % NC;
      const int t = min(start + kRound * ti + row, end - 1);   // past the end: a row that exists, zeroed below
      kr[i] = *reinterpret_cast<const u16x8*>(
          a.k_cache + ((int64_t)pg[(t >> a.log2_page) - page0] * a.page_size + (t & (a.page_size - 1))) * CK + 8 * ch);
    }
  };
  auto store = [&](int ti) {
    const int left = end - (start + kRound * ti);   // rows that exist
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int c = NT * i + tid, row = c / NC, ch = c % NC;
      *reinterpret_cast<u16x8*>(tile + RK * row + 16 * ch) = row < left ? kr[i] : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
  };

  float m_run = -1e30f, l_run = 0.f;   // finite start: no inf - inf
  f32x4 acc[NB];
#pragma unroll
  for (int m = 0; m < NB; ++m) acc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int nb = rp >> 4;

  load(0);
  for (int ti = 0; ti < ntile; ++ti) {
    __syncthreads();   // every wave is done with the previous tile
    store(ti);
    __syncthreads();
    if (ti + 1 < ntile) load(ti + 1);
    f32x4 d0 = f32x4{0.f, 0.f, 0.f, 0.f}, d1 = d0;
    const char* krow = tile + RK * (16 * w + l15) + 16 * lg;
#pragma unroll
    for (int st = 0; st < NK; st += 2) {
      d0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf8(*reinterpret_cast<const u16x8*>(krow + 64 * st)), bf8(qf[st]), d0, 0, 0, 0);
      d1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf8(*reinterpret_cast<const u16x8*>(krow + 64 * st + 64)), bf8(qf[st + 1]), d1, 0, 0, 0);
    }
    const int left = end - (start + kRound * ti + 16 * w + 4 * lg);   // this lane's 4 tokens that exist
    float sc[4];
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      sc[i] = i < left ? (d0[i] + d1[i]) * a.scale_log2 : -INFINITY;
      mx = fmaxf(mx, sc[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
    mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
    if (lg == 0) stat[hg][w][l15] = mx;
    __syncthreads();
    mx = m_run;
#pragma unroll
    for (int ww = 0; ww < 4; ++ww) mx = fmaxf(mx, stat[hg][ww][l15]);
    if (__any(mx > m_run)) {
      const float alpha = exp2f(m_run - mx);
      l_run *= alpha;
#pragma unroll
      for (int m = 0; m < NB; ++m) acc[m] *= alpha;
      m_run = mx;
    }
    f32x4 p;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      p[i] = exp2f(sc[i] - m_run);
      l_run += p[i];
    }
    ps[hg][w][lane] = __builtin_bit_cast(s16x4, __builtin_convertvector(p, bf16x4));
    __syncthreads();
    const char* vrow = tile + RK * (4 * lg + (l15 >> 2)) + 8 * (l15 & 3) + 32 * w;
#pragma unroll
    for (int st = 0; st < 2; ++st) {   // 32 tokens: two 16-token blocks, 4 tokens of each per lane
      const s16x8 pb = __builtin_shufflevector(ps[hg][2 * st][lane], ps[hg][2 * st + 1][lane], 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
      for (int m = 0; m < NB; ++m)
        if (4 * m + w < nb) {
          const char* v = vrow + RK * 32 * st + 128 * m;
          const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(v));
          const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(v + RK * 16));
          const s16x8 va = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
          acc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, va), __builtin_bit_cast(bf16x8, pb), acc[m], 0, 0, 0);
        }
    }
  }
  l_run += __shfl_xor(l_run, 16, kWave);
  l_run += __shfl_xor(l_run, 32, kWave);
  __syncthreads();
  if (lg == 0) stat[hg][w][l15] = l_run;   // the sum over this wave's tokens
  __syncthreads();
  if (h >= a.G) return;
  const float L = stat[hg][0][l15] + stat[hg][1][l15] + stat[hg][2][l15] + stat[hg][3][l15];
  const int64_t bh = (int64_t)b * a.G + h;
  float f = 1.f;
  if (ns_b == 1) f = (a.gate ? a.gate[bh] : 1.f) / L;
  const int64_t part = bh * a.num_splits + s;
#pragma unroll
  for (int m = 0; m < NB; ++m)
    if (4 * m + w < nb) {   // lane: head l15, dims 4 lg .. 4 lg + 3 of the block
      const int d = 16 * (4 * m + w) + 4 * lg;
      if (ns_b == 1) {
        const f32x4 o = acc[m] * f;
        *reinterpret_cast<uint2*>(a.out + (int64_t)b * a.o_ld + (int64_t)h * rp + d) = make_uint2(pack_bf2(o[0], o[1]), pack_bf2(o[2], o[3]));
      } else {
        *reinterpret_cast<f32x4*>(a.o_part + part * rp + d) = acc[m];
      }
    }
  if (ns_b > 1 && w == 0 && lg == 0) {
    a.ml_part[part * 2] = m_run;
    a.ml_part[part * 2 + 1] = L;
  }
}

int attn_latent_decode(const AttnDecode& a, int B, int rp, hipStream_t stream) {
  if (B == 0) return 0;
  if (a.Hkv != 1 || a.dkp % 64 || rp % 16 || rp > a.dkp || a.o_ld % 4 || a.G < 1 || a.page_size % 16 || a.max_pages > kMaxPages || a.num_splits < 1) return -1;
  const bool wide = a.G > 16;   // 32 heads share one staged tile
  const int hcs = wide ? (a.G + 31) / 32 : 1;
  const int grid = (B * a.num_splits + 7) / 8 * 8 * hcs;
#define OAMD_LAT(NK)                                                                                  \
  case 32 * NK:                                                                                       \
    if (wide) attn_latent_decode_kernel<NK, 2><<<grid, 512, 0, stream>>>(a, rp, B);                   \
    else attn_latent_decode_kernel<NK, 1><<<grid, 256, 0, stream>>>(a, rp, B);                        \
    break
  switch (a.dkp) {
    OAMD_LAT(4);
    OAMD_LAT(6);
    OAMD_LAT(8);
    OAMD_LAT(10);
    OAMD_LAT(12);
    OAMD_LAT(14);
    OAMD_LAT(16);
    OAMD_LAT(18);
    OAMD_LAT(20);
    default: return -2;
  }
#undef OAMD_LAT
  OAMD_LAUNCH_CHECK();
  if (a.num_splits > 1) return attn_combine(a, B, kRound, stream);
  return 0;
}

}  // namespace oamd
