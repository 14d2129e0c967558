// From a packed QKV projection to attention operands, one pass per token:
//   q, k  (+ bias) -> rotary positions on the first rot_pairs pairs of a head (dimension
//         2i with 2i + 1) -> divided by their root mean square over the head (no weight)
//   v     (+ bias) -> (1 - lam) v + lam v_first when the layer mixes values
//   k, v  -> paged cache (and, for a prefill, packed copies the attention reads)
// Any head size: a head occupies dkp (q, k) or dvp (v) columns, the true size rounded up
// by the loader with zero weights, so the tail is zero everywhere.
// Row layout: [q Hq x dkp | k Hkv x dkp | v Hkv x dvp | unused up to ncol].
//
// bf16 cache layout (read by attn_gd.hip): 16-token tiles. K tile [dkp/8 chunk][16 token]
// [8 dims]; V tile [dvp/32][4 token group][16 dims][2 half][4 token] (dim d = 32 b + 16 half
// + i). Every MFMA fragment of the decode kernel is then one contiguous 1 KiB wave access.
// fp32 cache: token rows.
#include "rows.h"

namespace oamd {

// GW lanes (a power of two) share a q / k head, each with CPT chunks of 8 dims (GW * CPT * 8 >= dkp);
// v is copied in 8-dim items. Grid (tokens, items / 256); consecutive tokens run on one XCD, so
// the pieces they write of one cache line meet in its L2.
template <typename T, int GW, int CPT>
__global__ void __launch_bounds__(256) qkv_heads_kernel(const QkvHeads a) {
  const int t = xcd_remap(blockIdx.x, gridDim.x);
  const int it = blockIdx.y * 256 + threadIdx.x;
  const int rot_items = (a.Hq + a.Hkv) * GW;
  const int vch = a.dvp >> 3;
  if (it >= rot_items + a.Hkv * vch) return;
  auto load = [&](int col, float (&v)[8]) {
    if (a.xp) {
      const float* p = a.xp + (int64_t)t * a.ncol + col;
      if constexpr (CPT == 1) {   // slabs: up to 8 requested before the first add
        float w[8][8];
#pragma unroll
        for (int s = 0; s < 8; ++s)
          if (s < a.S) ld8<float>(p + s * a.slab, w[s]);
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = w[0][j];
#pragma unroll
        for (int s = 1; s < 8; ++s)
          if (s < a.S) {
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] += w[s][j];
          }
      } else {
        ld8<float>(p, v);
      }
      for (int s = CPT == 1 ? 8 : 1; s < a.S; ++s) {
        float w[8];
        ld8<float>(p + s * a.slab, w);
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] += w[j];
      }
    } else {
      ld8<T>(static_cast<const T*>(a.row) + (int64_t)t * a.ncol + col, v);
    }
  };
  auto add_bias = [&](int col, float (&v)[8]) {
    if (a.bias) {
      float b[8];
      ld8<float>(a.bias + col, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] += b[j];
    }
  };
  const int64_t slot = a.slots ? a.slots[t] : -1;
  const int64_t page = slot >= 0 ? slot >> a.log2_page : 0;
  const int off = static_cast<int>(slot & ((1 << a.log2_page) - 1));

  if (it < rot_items) {
    const int h = it / GW, c0 = it % GW;   // head; chunks c0, c0 + GW, ...
    float x[CPT][8];
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int c = c0 + i * GW;
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] = 0.f;
      if (8 * c < a.dkp) load(h * a.dkp + 8 * c, x[i]);   // q heads then k heads: the same stride
    }
    int64_t p = 0;
    if (a.rot_pairs > 0) {
      p = a.pos[t];
      p = p < 0 ? 0 : (p >= a.max_pos ? a.max_pos - 1 : p);
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int c = c0 + i * GW;
      if (8 * c < a.dkp) {
        add_bias(h * a.dkp + 8 * c, x[i]);
        if (4 * c < a.rot_pairs) {
          const f32x4 cs = *reinterpret_cast<const f32x4*>(a.cos_t + p * a.rot_ld + 4 * c);
          const f32x4 sn = *reinterpret_cast<const f32x4*>(a.sin_t + p * a.rot_ld + 4 * c);
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (4 * c + j < a.rot_pairs) {
              const float u = x[i][2 * j], v = x[i][2 * j + 1];
              x[i][2 * j] = __builtin_fmaf(u, cs[j], -(v * sn[j]));
              x[i][2 * j + 1] = __builtin_fmaf(v, cs[j], u * sn[j]);
            }
        }
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += x[i][j] * x[i][j];
    }
    if (a.norm) {
      ss = group_sum<GW>(ss);
      const float rs = rsqrtf(ss / static_cast<float>(a.dk) + a.eps);
#pragma unroll
      for (int i = 0; i < CPT; ++i)
#pragma unroll
        for (int j = 0; j < 8; ++j) x[i][j] *= rs;
    }
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int c = c0 + i * GW;
      if (8 * c >= a.dkp) continue;
      if (h < a.Hq) {
        st8<T>(static_cast<T*>(a.q_out) + ((int64_t)t * a.Hq + h) * a.dkp + 8 * c, x[i]);
      } else {
        const int kh = h - a.Hq;
        if (a.k_out) st8<T>(static_cast<T*>(a.k_out) + ((int64_t)t * a.Hkv + kh) * a.dkp + 8 * c, x[i]);
        if (slot >= 0 && a.k_cache) {
          const int64_t head = (page * a.Hkv + kh) << a.log2_page;
          cache_k8<T>(static_cast<T*>(a.k_cache), head, off, a.dkp, c, x[i]);
        }
      }
    }
  } else {
    const int vi = it - rot_items;
    const int kh = vi / vch, c = vi % vch;
    const int col = (a.Hq + a.Hkv) * a.dkp + kh * a.dvp + 8 * c;
    float x[8];
    load(col, x);
    add_bias(col, x);
    const int64_t at = ((int64_t)t * a.Hkv + kh) * a.dvp + 8 * c;
    if (a.v_first) {
      float f[8];
      ld8<T>(static_cast<const T*>(a.v_first) + at, f);
      const float lam = *a.lam;
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] = (1.f - lam) * x[j] + lam * f[j];
    }
    if (a.v_out) st8<T>(static_cast<T*>(a.v_out) + at, x);
    if (slot >= 0 && a.v_cache) {
      const int64_t head = (page * a.Hkv + kh) << a.log2_page;
      cache_v8<T>(static_cast<T*>(a.v_cache), head, off, a.dvp, c, x);
    }
  }
}

template <typename T>
static int launch_qkv_heads(const QkvHeads& a, int tokens, hipStream_t stream) {
  // rows: two chunks per lane (two loads in flight); slabs: one chunk, its slabs in flight together
  const int cpt = a.xp ? 1 : 2;
  int gw = 1;
  while (gw * cpt * 8 < a.dkp) gw *= 2;
  const int items = (a.Hq + a.Hkv) * gw + a.Hkv * (a.dvp / 8);
  const dim3 grid(tokens, (items + 255) / 256);
#define OAMD_QKV(GW)                                                                   \
  case GW:                                                                             \
    if (cpt == 1) qkv_heads_kernel<T, GW, 1><<<grid, 256, 0, stream>>>(a);             \
    else qkv_heads_kernel<T, GW, 2><<<grid, 256, 0, stream>>>(a);                      \
    break
  switch (gw) {
    OAMD_QKV(1);
    OAMD_QKV(2);
    OAMD_QKV(4);
    OAMD_QKV(8);
    OAMD_QKV(16);
    OAMD_QKV(32);
    default: return -2;
  }
#undef OAMD_QKV
  OAMD_LAUNCH_CHECK();
  return 0;
}

int qkv_heads(const QkvHeads& a, int tokens, bool f32, hipStream_t stream) {
  if (tokens == 0) return 0;
  if (a.dkp % 8 || a.dvp % 8 || a.dkp > 256 || a.Hkv < 1 || a.Hq < 1) return -1;
  if (a.k_cache && !f32 && (a.dvp % 32 || a.log2_page < 4)) return -1;
  return f32 ? launch_qkv_heads<float>(a, tokens, stream) : launch_qkv_heads<bf16_t>(a, tokens, stream);
}

}  // namespace oamd
