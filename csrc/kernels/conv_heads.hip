// From a packed query | key | gate projection to attention operands of a layer with short causal
// convolutions, in one pass:
//   q, k   every channel: sum over the last `taps` tokens of its own weights (zeros before the
//          sequence's start), then per head x / sqrt(mean(x^2) + eps) * w
//   v      the convolved key before its norm
//   gate   sigmoid, one number per query head
//   k, v   -> paged cache (and, for a prefill, packed copies the attention reads)
// Row layout: [q Hq x dkp | k Hkv x dkp | gate Hq | unused up to ncol]; padding columns are zero.
//
// The recurrent state is the last taps - 1 projected rows of a sequence. It lives in the pages that
// hold those tokens: entry position % (taps - 1) of a page's tail [taps - 1][(Hq + Hkv) dkp], so it
// is allocated, shared (a common prompt prefix ends on a page's end) and freed with them. A prefill
// writes only the rows a later token can still ask for, each from one thread; a decode step reads
// and then overwrites an entry in the same thread.
#include "rows.h"

namespace oamd {

// GW lanes (a power of two) share a head, 8 dims each; a thread takes TM consecutive tokens, whose
// rows it loads once. TB: bound of a.taps. TM == 1: decode (earlier rows from the pages); else
// prefill (from the batch, and from the pages only before a sequence's first row).
template <typename T, int GW, int TB, int TM>
__global__ void __launch_bounds__(256) conv_heads_kernel(const ConvHeads a) {
  constexpr bool kDecode = TM == 1;
  const int t0 = xcd_remap(blockIdx.x, gridDim.x) * TM;
  const int it = blockIdx.y * 256 + threadIdx.x;
  const int lane = threadIdx.x & 63;
  const int items = (a.Hq + a.Hkv) * GW;
  const int R = a.taps - 1, C = (a.Hq + a.Hkv) * a.dkp;
  const int h = it / GW, c = it % GW, kh = h - a.Hq;
  const bool gated = it >= items;                 // gate items come after the heads
  const bool real = !gated && 8 * c < a.dkp;      // chunks past dkp: zero value columns
  const int col = h * a.dkp + 8 * c;
  T* tails = static_cast<T*>(a.tails);
  // u[TB - 1 + i]: projected row of token t0 + i; before them the rows of the batch just before t0
  Raw8<T> u[TB - 1 + TM];
#pragma unroll
  for (int i = 0; i < TB - 1 + TM; ++i) {
    u[i] = raw_zero<T>();
    const int t = t0 + i - (TB - 1);
    if (real && t < a.T && (i >= TB - 1 || (!kDecode && t >= 0 && i >= TB - 1 - R)))
      u[i] = raw_row8<T>(a.xp, a.row, a.S, a.slab, (int64_t)t * a.ncol + col);
  }
  Raw8<T> w[TB], nw = raw_zero<T>();
#pragma unroll
  for (int d = 0; d < TB; ++d) {
    w[d] = raw_zero<T>();
    if (real && d <= R) w[d] = raw_ld<T>(static_cast<const T*>(a.conv) + (int64_t)(R - d) * C + col);
  }
  if (real) nw = raw_ld<T>(static_cast<const T*>(kh < 0 ? a.qw : a.kw) + 8 * c);
  int64_t slot[TM], pos[TM];
#pragma unroll
  for (int i = 0; i < TM; ++i) {
    slot[i] = t0 + i < a.T ? a.slots[t0 + i] : -1;
    pos[i] = t0 + i < a.T ? a.pos[t0 + i] : 0;
  }
  int first = 0, last = 0x7fffffff;   // rows of the current sequence: first .. last - 1
  int64_t before = -1;                // page of the tokens before its first row
  int seq = -1;
  if (!kDecode) {   // the sequence of the first token: sequences that end at or before it
    seq = 0;
    for (int i = 0; i < a.num_seqs; i += 64)
      seq += __popcll(__ballot(i + lane < a.num_seqs && a.cu_seqlens[min(i + lane, a.num_seqs - 1) + 1] <= t0));
  }
  if (gated) {   // only now: every lane takes part in the search above
    const int gh = it - items;
    if (gh < a.Hq) {
#pragma unroll
      for (int i = 0; i < TM; ++i)
        if (t0 + i < a.T) {
          const float z = load_row1<T>(a.xp, a.row, a.S, a.slab, (int64_t)(t0 + i) * a.ncol + C + gh);
          a.gate[(int64_t)(t0 + i) * a.Hq + gh] = 1.f / (1.f + expf(-z));
        }
    }
    return;
  }
  auto enter = [&](int t) {   // past the last sequence: a padding row of a graph-captured prefill
    const bool in = seq < a.num_seqs;
    first = in ? a.cu_seqlens[seq] : t;
    last = in ? a.cu_seqlens[seq + 1] : 0x7fffffff;
    before = in && a.prev_page ? a.prev_page[seq] : -1;
  };
  if (!kDecode) enter(t0);
  float y[TM][8];
#pragma unroll
  for (int i = 0; i < TM; ++i) {
    const int t = t0 + i;
#pragma unroll
    for (int j = 0; j < 8; ++j) y[i][j] = 0.f;
    if (t >= a.T) continue;
    const int64_t p = pos[i];
    const int64_t page = slot[i] >= 0 ? slot[i] >> a.log2_page : 0;
    if (!kDecode)
      while (t >= last) {
        ++seq;
        enter(t);
      }
    const int own = kDecode ? 0 : t - first;   // rows of the same sequence before this one in the batch
    const bool keep = slot[i] >= 0 && R > 0 && (kDecode || (last != 0x7fffffff && t + R >= last));
    if (!real) continue;
#pragma unroll
    for (int d = TB - 1; d >= 1; --d) {
      if (d > R || p < d) continue;
      if (!kDecode && d <= own) {
#pragma unroll
        for (int j = 0; j < 8; ++j) y[i][j] = __builtin_fmaf(raw_at(w[d], j), raw_at(u[TB - 1 + i - d], j), y[i][j]);
        continue;
      }
      const int64_t q = p - d;
      int64_t pg = before;
      if (kDecode) {
        pg = page;
        if (q >> a.log2_page != p >> a.log2_page)
          pg = a.block_tables[(int64_t)t * a.max_pages + min((int)(q >> a.log2_page), a.max_pages - 1)];
      }
      if (pg < 0 || pg >= a.pages) continue;
      const Raw8<T> v = raw_ld<T>(tails + (pg * R + q % R) * C + col);
#pragma unroll
      for (int j = 0; j < 8; ++j) y[i][j] = __builtin_fmaf(raw_at(w[d], j), raw_at(v, j), y[i][j]);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) y[i][j] = __builtin_fmaf(raw_at(w[0], j), raw_at(u[TB - 1 + i], j), y[i][j]);
    if (keep) raw_st<T>(tails + (page * R + p % R) * C + col, u[TB - 1 + i]);
  }
  // four tokens of one aligned group of a page: a V tile keeps them side by side
  bool group = TM == 4 && sizeof(T) == 2 && slot[0] >= 0 && (slot[0] & 3) == 0;
#pragma unroll
  for (int i = 1; i < TM; ++i) group = group && slot[i] == slot[0] + i;
  if constexpr (TM == 4 && sizeof(T) == 2) {
    if (group && kh >= 0 && 8 * c < a.dvp) {
      const int64_t head = ((slot[0] >> a.log2_page) * a.Hkv + kh) << a.log2_page;
      const int off = static_cast<int>(slot[0] & ((1 << a.log2_page) - 1)), d0 = 8 * c;
      bf16_t* dst = static_cast<bf16_t*>(a.v_cache) + (head + (off & ~15)) * a.dvp +
                    (((d0 >> 5) * 4 + ((off & 15) >> 2)) * 16 + (d0 & 15)) * 8 + ((d0 >> 4) & 1) * 4;
#pragma unroll
      for (int j = 0; j < 8; ++j)
        *reinterpret_cast<uint2*>(dst + 8 * j) = make_uint2(pack_bf2(y[0][j], y[1][j]), pack_bf2(y[2][j], y[3][j]));
    }
  }
#pragma unroll
  for (int i = 0; i < TM; ++i) {
    const int t = t0 + i;
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) ss += y[i][j] * y[i][j];
    ss = group_sum<GW>(ss);
    if (t >= a.T) continue;
    const int64_t page = slot[i] >= 0 ? slot[i] >> a.log2_page : 0;
    const int off = static_cast<int>(slot[i] & ((1 << a.log2_page) - 1));
    const int64_t head = (page * a.Hkv + kh) << a.log2_page;
    if (kh >= 0 && 8 * c < a.dvp) {
      if (a.v_out) st8<T>(static_cast<T*>(a.v_out) + ((int64_t)t * a.Hkv + kh) * a.dvp + 8 * c, y[i]);
      if (slot[i] >= 0 && !group) cache_v8<T>(static_cast<T*>(a.v_cache), head, off, a.dvp, c, y[i]);
    }
    if (!real) continue;
    const float rs = 1.f / sqrtf(ss / static_cast<float>(a.dk) + a.eps);
#pragma unroll
    for (int j = 0; j < 8; ++j) y[i][j] = y[i][j] * rs * raw_at(nw, j);
    if (kh < 0) {
      st8<T>(static_cast<T*>(a.q_out) + ((int64_t)t * a.Hq + h) * a.dkp + 8 * c, y[i]);
    } else {
      if (a.k_out) st8<T>(static_cast<T*>(a.k_out) + ((int64_t)t * a.Hkv + kh) * a.dkp + 8 * c, y[i]);
      if (slot[i] >= 0) cache_k8<T>(static_cast<T*>(a.k_cache), head, off, a.dkp, c, y[i]);
    }
  }
}

template <typename T, int TB, int TM>
static int launch_conv_heads(const ConvHeads& a, hipStream_t stream) {
  int gw = 1;
  while (gw * 8 < a.dvp) gw *= 2;
  const int items = (a.Hq + a.Hkv) * gw + a.Hq;
  const dim3 grid((a.T + TM - 1) / TM, (items + 255) / 256);
  switch (gw) {
    case 4: conv_heads_kernel<T, 4, TB, TM><<<grid, 256, 0, stream>>>(a); break;
    case 8: conv_heads_kernel<T, 8, TB, TM><<<grid, 256, 0, stream>>>(a); break;
    case 16: conv_heads_kernel<T, 16, TB, TM><<<grid, 256, 0, stream>>>(a); break;
    case 32: conv_heads_kernel<T, 32, TB, TM><<<grid, 256, 0, stream>>>(a); break;
    default: return -2;
  }
  OAMD_LAUNCH_CHECK();
  return 0;
}

int conv_heads(const ConvHeads& a, bool f32, hipStream_t stream) {
  if (a.T == 0) return 0;
  if (a.dkp % 8 || a.dvp % 32 || a.dvp < a.dkp || a.dvp > 256 || a.Hkv < 1 || a.Hq < 1 || a.taps < 1 || a.taps > 8) return -1;
  if (a.k_cache == nullptr || a.v_cache == nullptr || a.slots == nullptr || a.log2_page < 4 || (a.taps > 1 && a.tails == nullptr)) return -1;
  if ((a.cu_seqlens == nullptr) == (a.block_tables == nullptr)) return -1;
#define OAMD_CONV(TB)                                                                                        \
  if (a.block_tables) return f32 ? launch_conv_heads<float, TB, 1>(a, stream) : launch_conv_heads<bf16_t, TB, 1>(a, stream); \
  return f32 ? launch_conv_heads<float, TB, 4>(a, stream) : launch_conv_heads<bf16_t, TB, 4>(a, stream)
  if (a.taps <= 4) { OAMD_CONV(4); }
  OAMD_CONV(8);
#undef OAMD_CONV
}

}  // namespace oamd
