// From a packed query | key | gate projection to attention operands of a layer with short causal
// convolutions, one pass per token:
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

// GW lanes (a power of two) share a head, each with CPT chunks of 8 dims. TB: bound of a.taps.
template <typename T, int GW, int CPT, int TB>
__global__ void __launch_bounds__(256) conv_heads_kernel(const ConvHeads a) {
  const int t = xcd_remap(blockIdx.x, gridDim.x);
  const int it = blockIdx.y * 256 + threadIdx.x;
  const int lane = threadIdx.x & 63;
  const int items = (a.Hq + a.Hkv) * GW;
  const int R = a.taps - 1, C = (a.Hq + a.Hkv) * a.dkp;
  const int64_t p = a.pos[t];
  const int64_t slot = a.slots ? a.slots[t] : -1;
  const int64_t page = slot >= 0 ? slot >> a.log2_page : 0;
  const int off = static_cast<int>(slot & ((1 << a.log2_page) - 1));
  // own rows before this one, the page of the tokens before the sequence's first row, rows still to come
  int own = 0;
  int64_t before = -1;
  bool keep = slot >= 0;
  if (a.cu_seqlens) {
    int s = 0;
    for (int i = 0; i < a.num_seqs; i += 64)
      s += __popcll(__ballot(i + lane < a.num_seqs && a.cu_seqlens[min(i + lane, a.num_seqs - 1) + 1] <= t));
    if (s < a.num_seqs) {   // else: a padding row of a graph-captured prefill
      own = t - a.cu_seqlens[s];
      if (a.prev_page) before = a.prev_page[s];
      keep = keep && t + R >= a.cu_seqlens[s + 1];
    }
  }
  if (it >= items) {
    const int h = it - items;
    if (h < a.Hq) {
      const float z = load_row1<T>(a.xp, a.row, a.S, a.slab, (int64_t)t * a.ncol + C + h);
      a.gate[(int64_t)t * a.Hq + h] = 1.f / (1.f + expf(-z));
    }
    return;
  }
  const int h = it / GW, c0 = it % GW;
  T* tails = static_cast<T*>(a.tails);
  float y[CPT][8];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const int c = c0 + i * GW;
#pragma unroll
    for (int j = 0; j < 8; ++j) y[i][j] = 0.f;
    if (8 * c >= a.dkp) continue;
    const int col = h * a.dkp + 8 * c;
    float u[TB][8];   // u[d]: the projected token d places back
#pragma unroll
    for (int d = 0; d < TB; ++d) {
#pragma unroll
      for (int j = 0; j < 8; ++j) u[d][j] = 0.f;
      if (d > R || p < d) continue;
      if (d == 0 || (a.cu_seqlens && d <= own)) {
        load_row8<T>(a.xp, a.row, a.S, a.slab, (int64_t)(t - d) * a.ncol + col, u[d]);
      } else {
        int64_t pg = before;
        if (a.block_tables) pg = a.block_tables[(int64_t)t * a.max_pages + min((int)((p - d) >> a.log2_page), a.max_pages - 1)];
        if (pg >= 0 && pg < a.pages) ld8<T>(tails + (pg * R + (p - d) % R) * C + col, u[d]);
      }
    }
#pragma unroll
    for (int d = TB - 1; d >= 0; --d)
      if (d <= R) {
        float w[8];
        ld8<float>(a.conv + (int64_t)(R - d) * C + col, w);
#pragma unroll
        for (int j = 0; j < 8; ++j) y[i][j] = __builtin_fmaf(w[j], u[d][j], y[i][j]);
      }
    if (keep && R > 0) st8<T>(tails + (page * R + p % R) * C + col, u[0]);
#pragma unroll
    for (int j = 0; j < 8; ++j) ss += y[i][j] * y[i][j];
  }
  ss = group_sum<GW>(ss);
  const float rs = 1.f / sqrtf(ss / static_cast<float>(a.dk) + a.eps);
  const float* nw = h < a.Hq ? a.qw : a.kw;
  const int kh = h - a.Hq;
  const int64_t head = (page * a.Hkv + kh) << a.log2_page;
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const int c = c0 + i * GW;
    if (kh >= 0 && 8 * c < a.dvp) {   // value columns past dkp: zeros
      if (a.v_out) st8<T>(static_cast<T*>(a.v_out) + ((int64_t)t * a.Hkv + kh) * a.dvp + 8 * c, y[i]);
      if (slot >= 0) cache_v8<T>(static_cast<T*>(a.v_cache), head, off, a.dvp, c, y[i]);
    }
    if (8 * c >= a.dkp) continue;
    float w[8];
    ld8<float>(nw + 8 * c, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) y[i][j] = y[i][j] * rs * w[j];
    if (kh < 0) {
      st8<T>(static_cast<T*>(a.q_out) + ((int64_t)t * a.Hq + h) * a.dkp + 8 * c, y[i]);
    } else {
      if (a.k_out) st8<T>(static_cast<T*>(a.k_out) + ((int64_t)t * a.Hkv + kh) * a.dkp + 8 * c, y[i]);
      if (slot >= 0) cache_k8<T>(static_cast<T*>(a.k_cache), head, off, a.dkp, c, y[i]);
    }
  }
}

template <typename T, int TB>
static int launch_conv_heads(const ConvHeads& a, int tokens, hipStream_t stream) {
  int gw = 1;
  while (gw * 8 < a.dvp) gw *= 2;   // one chunk per lane: its taps are in flight together
  const int items = (a.Hq + a.Hkv) * gw + a.Hq;
  const dim3 grid(tokens, (items + 255) / 256);
  switch (gw) {
    case 4: conv_heads_kernel<T, 4, 1, TB><<<grid, 256, 0, stream>>>(a); break;
    case 8: conv_heads_kernel<T, 8, 1, TB><<<grid, 256, 0, stream>>>(a); break;
    case 16: conv_heads_kernel<T, 16, 1, TB><<<grid, 256, 0, stream>>>(a); break;
    case 32: conv_heads_kernel<T, 32, 1, TB><<<grid, 256, 0, stream>>>(a); break;
    default: return -2;
  }
  OAMD_LAUNCH_CHECK();
  return 0;
}

int conv_heads(const ConvHeads& a, int tokens, bool f32, hipStream_t stream) {
  if (tokens == 0) return 0;
  if (a.dkp % 8 || a.dvp % 32 || a.dvp < a.dkp || a.dvp > 256 || a.Hkv < 1 || a.Hq < 1 || a.taps < 1 || a.taps > 8) return -1;
  if (a.k_cache == nullptr || a.v_cache == nullptr || a.log2_page < 4 || (a.taps > 1 && a.tails == nullptr)) return -1;
  if (a.taps <= 4) return f32 ? launch_conv_heads<float, 4>(a, tokens, stream) : launch_conv_heads<bf16_t, 4>(a, tokens, stream);
  return f32 ? launch_conv_heads<float, 8>(a, tokens, stream) : launch_conv_heads<bf16_t, 8>(a, tokens, stream);
}

}  // namespace oamd
