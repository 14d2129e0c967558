// Causal flash attention for prefill with any query/key size and any value size (each up to
// 256), packed variable-length sequences, GQA: the swapped-operand 32x32 MFMA structure of
// attn_prefill.hip with the head sizes as template parameters and the group size at run time.
//
// A work item is 128 query rows of one sequence; grid (items, key/value head x head chunk,
// sub-block). A head chunk is GC <= 4 of the G query heads that share a key/value head (GC
// divides G), a workgroup is 4 waves: wave w takes head w % GC and 32 query rows of row block
// w / GC (4 / GC row blocks), so one staged K / V tile feeds GC heads. Layers with different
// head counts share one work list.
// Per 64-key tile: S^T = K Q^T (query row on the lane, so the softmax is lane-local), then
// O^T += V^T P^T with P straight from the accumulator registers and V^T through the
// transposing LDS read. The rescale is deferred (a running maximum is kept until a tile
// raises it by more than 8 in log2 units).
// seq_pfx: keys of a shared prompt prefix (rows of pk / pv) come before a sequence's own.
// window: tiles that no row of the workgroup sees are never loaded.
#include "attn_gd.h"

namespace oamd {

using namespace gd;

namespace {

__device__ __forceinline__ s16x4 tr16(const char* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(p));
}

}  // namespace

// DK, DV: instantiated sizes >= the stored sizes dkp, dvp (the rest is zero in LDS)
template <int DK, int DV>
__global__ void __launch_bounds__(256, (DK + DV <= 320) ? 2 : 1) attn_gd_prefill_kernel(const AttnPrefill a) {
  constexpr int BK = 64, RK = 2 * DK + 16;       // K rows padded by 16 B: conflict-free row reads
  constexpr int RV = DV <= 128 ? 256 : 512;      // V rows: the 16-chunk swizzle below needs 256-B rows
  constexpr int CK = DK / 8, CV = DV / 8;
  constexpr int NCK = BK * CK / 256, NCV = BK * CV / 256;
  constexpr int KS = DK / 16, DB = DV / 32;
  __shared__ __attribute__((aligned(16))) char Ks[BK * RK];
  __shared__ __attribute__((aligned(16))) char Vs[BK * RV];

  int wi = blockIdx.x, by = blockIdx.y, bz = blockIdx.z;
  if (gridDim.y % 8 == 0) {   // a head's workgroups on one XCD, an item's sub-blocks next to each other
    const int L = blockIdx.x + gridDim.x * (blockIdx.y + gridDim.y * blockIdx.z);
    const int j = L >> 3;
    bz = j % gridDim.z;
    wi = j / gridDim.z % gridDim.x;
    by = j / gridDim.z / gridDim.x * 8 + (L & 7);
  }
  const int seq = a.work_seq[wi];
  if (seq < 0) return;   // padding item of a graph-captured prefill (fixed grid)
  const int GC = a.gc, nch = a.G / GC;
  const int kvh = by / nch, hc = by % nch;
  const int RG = 4 / GC, BQ = 32 * RG;
  const int s0 = a.cu_seqlens[seq];
  const int slen = a.cu_seqlens[seq + 1] - s0;
  const int q0 = a.work_q0[wi] + bz * BQ;
  if (q0 >= slen) return;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r32 = lane & 31, h = lane >> 5;
  const int hq = kvh * a.G + hc * GC + (w % GC);
  const int rbase = q0 + 32 * (w / GC);
  const int qrow = rbase + r32;
  const bool wave_used = w < GC * RG;
  const int Hq = a.Hkv * a.G;

  u16x8 qb[KS];
#pragma unroll
  for (int s = 0; s < KS; ++s)
    qb[s] = (wave_used && qrow < slen && 16 * s + 8 * h < a.dkp)
                ? *reinterpret_cast<const u16x8*>(a.q + ((int64_t)(s0 + qrow) * Hq + hq) * a.dkp + 16 * s + 8 * h)
                : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
  f32x16 oacc[DB];
#pragma unroll
  for (int dd = 0; dd < DB; ++dd)
#pragma unroll
    for (int i = 0; i < 16; ++i) oacc[dd][i] = 0.f;
  float mrow = -INFINITY, lpart = 0.f;

  const int kend = min(slen, q0 + BQ);
  const int pl = a.seq_pfx != nullptr ? a.seq_pfx[seq] : 0;
  const int npt = (pl + BK - 1) / BK;
  const int ntiles = npt + (kend + BK - 1) / BK;
  // first tile with a key that the first row sees (keys count from the prefix's start)
  const int lo = pl + q0 - a.window + 1;
  const int kt0 = lo <= 0 ? 0 : lo < pl ? lo / BK : npt + (lo - pl) / BK;
  const bool active = wave_used && rbase < slen;
  const int wend = min(slen, rbase + 32);   // own keys this wave can see: < wend

  const int gi = lane & 15, g = lane >> 4;
  const int trq = gi >> 2, trp = gi & 3;
  auto v_img = [](int r, int ch) { return RV * r + 16 * ((ch & 16) | ((ch & 15) ^ (((r & 3) << 2) | ((r >> 2) & 3)))); };

  u16x8 kr[NCK], vr[NCV];
  // rows of key tile kt: prefix rows (kt < npt) or own rows of tile kt - npt
  auto row_of = [&](int kt, int key, bool& ok) -> int64_t {
    if (kt < npt) {
      ok = kt * BK + key < pl;
      return kt * BK + key;
    }
    ok = (kt - npt) * BK + key < slen;
    return (int64_t)s0 + (kt - npt) * BK + key;
  };
  auto load_tile = [&](int kt) {
    const bf16_t* kp = kt < npt ? a.pk : a.k;
    const bf16_t* vp = kt < npt ? a.pv : a.v;
#pragma unroll
    for (int r = 0; r < NCK; ++r) {
      const int c = tid + r * 256, key = c / CK, ch = c % CK;
      bool ok;
      const int64_t row = row_of(kt, key, ok);
      kr[r] = u16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (ok && 8 * ch < a.dkp) kr[r] = *reinterpret_cast<const u16x8*>(kp + (row * a.Hkv + kvh) * a.dkp + 8 * ch);
    }
#pragma unroll
    for (int r = 0; r < NCV; ++r) {
      const int c = tid + r * 256, key = c / CV, ch = c % CV;
      bool ok;
      const int64_t row = row_of(kt, key, ok);
      vr[r] = u16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (ok && 8 * ch < a.dvp) vr[r] = *reinterpret_cast<const u16x8*>(vp + (row * a.Hkv + kvh) * a.dvp + 8 * ch);
    }
  };
  auto store_tile = [&]() {
#pragma unroll
    for (int r = 0; r < NCK; ++r) {
      const int c = tid + r * 256, key = c / CK, ch = c % CK;
      *reinterpret_cast<u16x8*>(Ks + RK * key + 16 * ch) = kr[r];
    }
#pragma unroll
    for (int r = 0; r < NCV; ++r) {
      const int c = tid + r * 256, key = c / CV, ch = c % CV;
      *reinterpret_cast<u16x8*>(Vs + v_img(key, ch)) = vr[r];
    }
  };

  load_tile(kt0);
  for (int kt = kt0; kt < ntiles; ++kt) {
    const int kb = (kt - npt) * BK;   // own-key coordinates (negative: a prefix tile)
    __syncthreads();
    store_tile();
    __syncthreads();
    if (!active || kb >= wend) {      // wave-uniform: no visible key for this wave
      if (kt + 1 < ntiles) load_tile(kt + 1);
      continue;
    }
    f32x16 sacc[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
#pragma unroll
      for (int i = 0; i < 16; ++i) sacc[b][i] = 0.f;
      const char* krow = Ks + RK * (32 * b + r32) + 16 * h;
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const u16x8 ka = *reinterpret_cast<const u16x8*>(krow + 32 * s);
        sacc[b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(bf8(ka), bf8(qb[s]), sacc[b], 0, 0, 0);
      }
    }
    if (kt + 1 < ntiles) load_tile(kt + 1);   // in flight during softmax + P.V
    // register i of block b is key kb + 32b + (i&3) + 8(i>>2) + 4h
    const bool ptile = kb < 0;
    const int pend = pl - kt * BK;
    const int wlo = qrow - a.window - (ptile ? kt * BK - pl : kb);   // tile keys up to here are out of the row's window
    const bool mask = (ptile ? (pend < BK) : ((kb + BK > rbase + 1) || (kb + BK > slen))) ||
                      rbase + 31 - a.window >= (ptile ? kt * BK - pl : kb);
    float mx = -INFINITY;
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        float sv = sacc[b][i] * a.scale_log2;
        if (mask) {
          const int j = 32 * b + (i & 3) + 8 * (i >> 2) + 4 * h;
          if ((ptile ? (j >= pend) : (kb + j > qrow || kb + j >= slen)) || j <= wlo) sv = -INFINITY;
        }
        sacc[b][i] = sv;
        mx = fmaxf(mx, sv);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
    float mnew = fmaxf(mrow, mx);
    const bool rescale = mrow == -INFINITY || mnew > mrow + 8.f;
    if (!rescale) mnew = mrow;
    const float msafe = (mnew == -INFINITY) ? 0.f : mnew;
    const float alpha = rescale ? exp2f(mrow - msafe) : 1.f;
    mrow = mnew;
    float rs = 0.f;
    u16x8 pb[2][2];
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        f32x8 p;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          p[j] = exp2f(sacc[b][8 * s + j] - msafe);
          rs += p[j];
        }
        pb[b][s] = __builtin_bit_cast(u16x8, __builtin_convertvector(p, bf16x8));
      }
    lpart = lpart * alpha + rs;
    if (rescale) {
#pragma unroll
      for (int dd = 0; dd < DB; ++dd)
#pragma unroll
        for (int i = 0; i < 16; ++i) oacc[dd][i] *= alpha;
    }
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        const int r0 = 32 * b + 16 * s + 4 * h + trq;
#pragma unroll
        for (int dd = 0; dd < DB; ++dd) {
          const int d = 32 * dd + 16 * (g & 1) + 4 * trp;
          const s16x4 lo = tr16(Vs + v_img(r0, d >> 3) + 8 * ((d >> 2) & 1));
          const s16x4 hi = tr16(Vs + v_img(r0 + 8, d >> 3) + 8 * ((d >> 2) & 1));
          const s16x8 va = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
          oacc[dd] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, va), bf8(pb[b][s]), oacc[dd], 0, 0, 0);
        }
      }
  }
  if (!active) return;
  const float lsum = lpart + __shfl_xor(lpart, 32, kWave);
  if (qrow >= slen) return;
  float inv = lsum > 0.f ? 1.f / lsum : 0.f;
  if (a.gate) inv *= a.gate[(int64_t)(s0 + qrow) * Hq + hq];
  bf16_t* dst = a.o + (int64_t)(s0 + qrow) * a.o_ld + hq * a.dvp;
  // register i of block dd is dim 32 dd + (i&3) + 8(i>>2) + 4h
#pragma unroll
  for (int dd = 0; dd < DB; ++dd)
    if (32 * dd < a.dvp) {
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        u16x4 st;
#pragma unroll
        for (int e = 0; e < 4; ++e) st[e] = f2bf(oacc[dd][4 * c + e] * inv);
        *reinterpret_cast<u16x4*>(dst + 32 * dd + 8 * c + 4 * h) = st;
      }
    }
}

template <int DK>
static int launch_dv(const AttnPrefill& a, dim3 grid, hipStream_t stream) {
  switch (dim_bin(a.dvp)) {
    case 32: attn_gd_prefill_kernel<DK, 32><<<grid, 256, 0, stream>>>(a); break;
    case 64: attn_gd_prefill_kernel<DK, 64><<<grid, 256, 0, stream>>>(a); break;
    case 96: attn_gd_prefill_kernel<DK, 96><<<grid, 256, 0, stream>>>(a); break;
    case 128: attn_gd_prefill_kernel<DK, 128><<<grid, 256, 0, stream>>>(a); break;
    case 192:
    case 256: attn_gd_prefill_kernel<DK, 256><<<grid, 256, 0, stream>>>(a); break;
    default: return -2;
  }
  OAMD_LAUNCH_CHECK();
  return 0;
}

int attn_gd_prefill(const AttnPrefill& a, int num_work, hipStream_t stream) {
  if (num_work == 0) return 0;
  if (a.dkp % 8 || a.dvp % 32 || a.G < 1 || a.gc < 1 || a.gc > 4 || a.G % a.gc || a.window < 1) return -1;
  const int rg = 4 / a.gc, sub = 4 / rg;   // 32 rg rows per workgroup, 128 per work item
  const dim3 grid(num_work, a.Hkv * (a.G / a.gc), sub);
  switch (dim_bin(a.dkp)) {
    case 32: return launch_dv<32>(a, grid, stream);
    case 64: return launch_dv<64>(a, grid, stream);
    case 96: return launch_dv<96>(a, grid, stream);
    case 128: return launch_dv<128>(a, grid, stream);
    case 192: return launch_dv<192>(a, grid, stream);
    case 256: return launch_dv<256>(a, grid, stream);
    default: return -2;
  }
}

}  // namespace oamd
