// Paged decode attention over latent rows: every query head of a sequence reads the same cached row
// [c (rp) | rotated part | 0 .. ck), its score is the product with the whole row and its value is c.
//
// Workgroup = (sequence, split, 16 query heads); 4 waves, each walking its own 16-token tiles with no
// barrier between them. A tile's rows are loaded once, contiguous, held in registers while the
// previous tile is worked on, and stored to the wave's own LDS block, from which both products read:
//   S = K Q^T     v_mfma_f32_16x16x32_bf16, A = rows (tokens x dims), B = q (one head per column)
//   O^T += V^T P  v_mfma_f32_16x16x16_bf16, A = the same rows through the transposing LDS read, B = P
//                 as S left it in the registers; a lane's column is one head, so the softmax is
//                 lane-local up to two shuffles
// Rows are padded by 16 bytes in LDS, which spreads both access patterns over the banks.
// Head chunks of one (sequence, split) run on one XCD and share its L2. Split sequences leave fp32
// partials for the combine kernel of attn_gd_decode.hip.
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

// NK: 32-dim steps of a row, ck = 32 NK
template <int NK>
__global__ void __launch_bounds__(256, 1) attn_latent_decode_kernel(const AttnDecode a, int rp, int B) {
  constexpr int CK = 32 * NK, RK = 2 * CK + 16, NC = CK / 8;
  __shared__ int pg[kMaxPages];
  __shared__ __attribute__((aligned(16))) char tiles[4 * 16 * RK];
  __shared__ float mls[4][16][2];
  const int hcs = (a.G + 15) / 16;
  const int items = B * a.num_splits;
  const int j = blockIdx.x >> 3;
  const int item = (j / hcs) * 8 + (blockIdx.x & 7);
  if (item >= items) return;
  const int b = item / a.num_splits, s = item % a.num_splits, h0 = (j % hcs) * 16;
  const int nh = min(16, a.G - h0);
  const int len = min(a.seq_lens[b], a.max_pages * a.page_size);
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, lg = lane >> 4;
  bf16_t* orow = a.out + (int64_t)b * a.o_ld + h0 * rp;
  if (len <= 0) {   // padding row: zeros, written once
    if (s == 0)
      for (int e = tid; e < nh * rp; e += 256) orow[e] = 0;
    return;
  }
  const int per = latent_split(len, a.num_splits);
  const int start = s * per;
  if (start >= len) return;
  const int end = min(len, start + per);
  const int ns_b = (len + per - 1) / per;
  const int ntile = (end - start + 15) / 16;

  const int page0 = start >> a.log2_page;
  const int npg = ((end - 1) >> a.log2_page) - page0 + 1;
  const int* btb = a.block_tables + (int64_t)b * a.max_pages + page0;
  for (int i = tid; i < npg; i += 256) pg[i] = btb[i];

  u16x8 qf[NK];
#pragma unroll
  for (int st = 0; st < NK; ++st)
    qf[st] = l15 < nh ? *reinterpret_cast<const u16x8*>(a.q + ((int64_t)b * a.G + h0 + l15) * CK + 32 * st + 8 * lg)
                      : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
  __syncthreads();

  char* tile = tiles + w * 16 * RK;
  const int nb = rp >> 4;
  u16x8 kr[NK];
  auto load = [&](int ti) {   // 16 rows of one page, contiguous
    const int t0 = start + 16 * ti;
    const bf16_t* src = a.k_cache + ((int64_t)pg[(t0 >> a.log2_page) - page0] * a.page_size + (t0 & (a.page_size - 1))) * CK;
#pragma unroll
    for (int i = 0; i < NK; ++i) kr[i] = *reinterpret_cast<const u16x8*>(src + (64 * i + lane) * 8);
  };
  auto store = [&](int ti) {
    const int left = end - (start + 16 * ti);   // rows that exist
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int c = 64 * i + lane, row = c / NC, ch = c % NC;
      // stale rows past the end must not reach the value product, not even times 0
      *reinterpret_cast<u16x8*>(tile + RK * row + 16 * ch) = row < left ? kr[i] : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
    }
  };
  auto wave_sync = [&]() {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
  };

  float m_run = -1e30f, l_run = 0.f;   // finite start: no inf - inf
  f32x4 acc[2 * NK];
#pragma unroll
  for (int m = 0; m < 2 * NK; ++m) acc[m] = f32x4{0.f, 0.f, 0.f, 0.f};

  if (w < ntile) load(w);
  for (int ti = w; ti < ntile; ti += 4) {
    store(ti);
    if (ti + 4 < ntile) load(ti + 4);
    wave_sync();
    f32x4 d0 = f32x4{0.f, 0.f, 0.f, 0.f}, d1 = d0;
    const char* krow = tile + RK * l15 + 16 * lg;
#pragma unroll
    for (int st = 0; st < NK; st += 2) {
      d0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf8(*reinterpret_cast<const u16x8*>(krow + 64 * st)), bf8(qf[st]), d0, 0, 0, 0);
      d1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf8(*reinterpret_cast<const u16x8*>(krow + 64 * st + 64)), bf8(qf[st + 1]), d1, 0, 0, 0);
    }
    const int left = end - (start + 16 * ti + 4 * lg);   // this lane's 4 tokens that exist
    float sc[4];
    float mx = m_run;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      sc[i] = i < left ? (d0[i] + d1[i]) * a.scale_log2 : -INFINITY;
      mx = fmaxf(mx, sc[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
    mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
    if (__any(mx > m_run)) {
      const float alpha = exp2f(m_run - mx);
      l_run *= alpha;
#pragma unroll
      for (int m = 0; m < 2 * NK; ++m) acc[m] *= alpha;
      m_run = mx;
    }
    f32x4 p;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      p[i] = exp2f(sc[i] - m_run);
      l_run += p[i];
    }
    const s16x4 pb = __builtin_bit_cast(s16x4, __builtin_convertvector(p, bf16x4));
    const char* vrow = tile + RK * (4 * lg + (l15 >> 2)) + 8 * (l15 & 3);
#pragma unroll
    for (int m = 0; m < 2 * NK; ++m)
      if (m < nb) {
        const s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(vrow + 32 * m));
        acc[m] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(v, pb, acc[m], 0, 0, 0);
      }
    wave_sync();   // the next tile overwrites this one
  }
  l_run += __shfl_xor(l_run, 16, kWave);
  l_run += __shfl_xor(l_run, 32, kWave);
  if (lg == 0) {
    mls[w][l15][0] = m_run;
    mls[w][l15][1] = l_run;
  }
  __syncthreads();   // every wave is done with its tile: the block becomes the merge buffer
  float* red = reinterpret_cast<float*>(tiles);   // [16][rp + 4]
  const int rld = rp + 4;
  float M = mls[0][l15][0];
#pragma unroll
  for (int ww = 1; ww < 4; ++ww) M = fmaxf(M, mls[ww][l15][0]);
  const float f = exp2f(m_run - M);
#pragma unroll
  for (int ww = 0; ww < 4; ++ww) {
    if (w == ww) {
#pragma unroll
      for (int m = 0; m < 2 * NK; ++m)
        if (m < nb) {
          f32x4* dst = reinterpret_cast<f32x4*>(red + l15 * rld + 16 * m + 4 * lg);
          *dst = ww == 0 ? acc[m] * f : *dst + acc[m] * f;
        }
    }
    __syncthreads();
  }
  for (int e = tid; e < nh * rp; e += 256) {
    const int h = e / rp, d = e % rp;
    float Mh = mls[0][h][0], L = 0.f;
#pragma unroll
    for (int ww = 1; ww < 4; ++ww) Mh = fmaxf(Mh, mls[ww][h][0]);
#pragma unroll
    for (int ww = 0; ww < 4; ++ww) L += exp2f(mls[ww][h][0] - Mh) * mls[ww][h][1];
    const float o = red[h * rld + d];
    const int64_t bh = (int64_t)b * a.G + h0 + h;
    if (ns_b == 1) {
      const float g = a.gate ? a.gate[bh] : 1.f;
      orow[e] = f2bf(L > 0.f ? o * g / L : 0.f);
    } else {
      a.o_part[(bh * a.num_splits + s) * rp + d] = o;
      if (d == 0) {
        a.ml_part[(bh * a.num_splits + s) * 2] = Mh;
        a.ml_part[(bh * a.num_splits + s) * 2 + 1] = L;
      }
    }
  }
}

int attn_latent_decode(const AttnDecode& a, int B, int rp, hipStream_t stream) {
  if (B == 0) return 0;
  if (a.Hkv != 1 || a.dkp % 64 || rp % 16 || rp > a.dkp || a.G < 1 || a.page_size % 16 || a.max_pages > kMaxPages || a.num_splits < 1) return -1;
  const int hcs = (a.G + 15) / 16;
  const int grid = (B * a.num_splits + 7) / 8 * 8 * hcs;
#define OAMD_LAT(NK) case 32 * NK: attn_latent_decode_kernel<NK><<<grid, 256, 0, stream>>>(a, rp, B); break
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
