// Pieces of latent attention: keys and values of all heads are products of one low-rank row per
// token, which is all the cache keeps.
//   latent_rows   projection [query latent | latent | rotated key part | gate] -> normed query
//                 latent, the cached row [c (rp) | rotated key part | 0 .. ck), sigmoid gates
//   rotate_heads  rotary positions on the last rot dims of every query head, first half paired
//                 with the second; sums split-K slabs on the way
//   head_gemm     one small product per head, Y_h = X_h W_h^T: into the latent space before a
//                 decode step's attention and out of it afterwards
#include "rows.h"

namespace oamd {

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

}  // namespace

// NT threads per token (256: a workgroup, for few tokens; 64: a wave); a segment of n padded columns is
// 8-column chunks tid, tid + NT, ...
template <typename T, int NT, int MAXC>
__global__ void __launch_bounds__(256) latent_rows_kernel(const LatentRows a, int tokens) {
  __shared__ float scratch[8];
  const int t = xcd_remap(blockIdx.x, gridDim.x) * (256 / NT) + threadIdx.x / NT, tid = threadIdx.x % NT;
  if (NT == 64 && t >= tokens) return;   // whole waves, and no barrier follows
  const int64_t row = (int64_t)t * a.ncol;
  const int nq = a.qp >> 3, nc = a.lat ? a.rp >> 3 : 0;
  float x[MAXC][8];
  float sq = 0.f, sc = 0.f;
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int ch = tid + NT * i;   // query latent chunks, then latent chunks
    if (ch >= nq + nc) continue;
    load_row8<T>(a.xp, a.row, a.S, a.slab, row + 8 * ch, x[i]);
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) s += x[i][j] * x[i][j];
    if (ch < nq) sq += s;
    else sc += s;
  }
  const int64_t slot = nc && a.slots ? a.slots[t] : -1;
  T* cq = static_cast<T*>(a.cq) + (int64_t)t * a.qp;
  T* lat = nc ? static_cast<T*>(a.lat) + (int64_t)t * a.ck : nullptr;
  T* kept = slot >= 0 ? static_cast<T*>(a.cache) + slot * a.ck : nullptr;   // page rows are contiguous: slot = page * P + token
  const int after = a.qp + (nc ? a.rp + a.rotp : 0);
  if (nc) {
    const int half = a.rot >> 1;
    int64_t p = a.pos[t];
    p = p < 0 ? 0 : (p >= a.max_pos ? a.max_pos - 1 : p);
    for (int i = tid; i < half; i += NT) {
      const int64_t at = row + a.qp + a.rp + i;
      const float u = load_row1<T>(a.xp, a.row, a.S, a.slab, at), v = load_row1<T>(a.xp, a.row, a.S, a.slab, at + half);
      float o1, o2;
      rope_pair(u, v, a.cos_t[p * a.rot_ld + i], a.sin_t[p * a.rot_ld + i], o1, o2);
      st1<T>(lat + a.rp + i, o1);
      st1<T>(lat + a.rp + half + i, o2);
      if (kept) {
        st1<T>(kept + a.rp + i, o1);
        st1<T>(kept + a.rp + half + i, o2);
      }
    }
    for (int i = a.rp + a.rot + tid; i < a.ck; i += NT) {
      st1<T>(lat + i, 0.f);
      if (kept) st1<T>(kept + i, 0.f);
    }
  }
  for (int h = tid; h < a.H; h += NT)
    a.gate[(int64_t)t * a.H + h] = 1.f / (1.f + expf(-load_row1<T>(a.xp, a.row, a.S, a.slab, row + after + h)));
  sq = wave_sum(sq);   // both sums in one exchange
  sc = wave_sum(sc);
  if constexpr (NT == 256) {
    if ((tid & 63) == 0) {
      scratch[tid >> 6] = sq;
      scratch[4 + (tid >> 6)] = sc;
    }
    __syncthreads();
    sq = scratch[0] + scratch[1] + scratch[2] + scratch[3];
    sc = scratch[4] + scratch[5] + scratch[6] + scratch[7];
  }
  const float rq = 1.f / sqrtf(sq / static_cast<float>(a.q_rank) + a.eps);
  const float rc = nc ? 1.f / sqrtf(sc / static_cast<float>(a.kv_rank) + a.eps) : 0.f;
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int ch = tid + NT * i;
    if (ch >= nq + nc) continue;
    float w[8];
    ld8<float>(ch < nq ? a.qw + 8 * ch : a.cw + 8 * (ch - nq), w);
    const float r = ch < nq ? rq : rc;
#pragma unroll
    for (int j = 0; j < 8; ++j) x[i][j] = x[i][j] * r * w[j];
    if (ch < nq) {
      st8<T>(cq + 8 * ch, x[i]);
    } else {
      st8<T>(lat + 8 * (ch - nq), x[i]);
      if (kept) st8<T>(kept + 8 * (ch - nq), x[i]);
    }
  }
}

int latent_rows(const LatentRows& a, int tokens, bool f32, hipStream_t stream) {
  if (tokens == 0) return 0;
  if (a.qp % 8 || a.rp % 8 || a.rot % 2 || a.rot > a.rotp || a.rp + a.rot > a.ck || a.H < 1) return -1;
  const int chunks = a.qp / 8 + (a.lat ? a.rp / 8 : 0);
  if (chunks > 1024) return -2;
  const bool wave = tokens >= 1024;
#define OAMD_LATENT(T)                                                                                  \
  if (wave && chunks <= 256) latent_rows_kernel<T, 64, 4><<<(tokens + 3) / 4, 256, 0, stream>>>(a, tokens);  \
  else if (chunks <= 256) latent_rows_kernel<T, 256, 1><<<tokens, 256, 0, stream>>>(a, tokens);         \
  else latent_rows_kernel<T, 256, 4><<<tokens, 256, 0, stream>>>(a, tokens)
  if (f32) { OAMD_LATENT(float); } else { OAMD_LATENT(bf16_t); }
#undef OAMD_LATENT
  OAMD_LAUNCH_CHECK();
  return 0;
}

// Rows [T][H][dp], a head = [d unrotated | rot | padding]. Rows mode (xp == nullptr) is in place and
// touches the rotated part only; a thread turns V neighbouring pairs. Slabs: every column is summed.
template <typename T, int V>
__global__ void __launch_bounds__(256) rotate_rows_kernel(const RotateHeads a, int64_t items) {
  const int half = a.rot >> 1, per = half / V;
  for (int64_t it = blockIdx.x * 256LL + threadIdx.x; it < items; it += gridDim.x * 256LL) {
    const int64_t th = it / per;
    const int i = (int)(it - th * per) * V;
    const int64_t t = th / a.H;
    int64_t p = a.pos[t];
    p = p < 0 ? 0 : (p >= a.max_pos ? a.max_pos - 1 : p);
    T* x = static_cast<T*>(a.q) + th * a.dp + a.d + i;
    const float* cs = a.cos_t + p * a.rot_ld + i;
    const float* sn = a.sin_t + p * a.rot_ld + i;
    if constexpr (V == 8) {
      float u[8], v[8];
      ld8<T>(x, u);
      ld8<T>(x + half, v);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        float o1, o2;
        rope_pair(u[j], v[j], cs[j], sn[j], o1, o2);
        u[j] = o1;
        v[j] = o2;
      }
      st8<T>(x, u);
      st8<T>(x + half, v);
    } else {
      float u[1], v[1], o1, o2;
      if constexpr (sizeof(T) == 4) {
        u[0] = x[0];
        v[0] = x[half];
      } else {
        u[0] = bf2f(x[0]);
        v[0] = bf2f(x[half]);
      }
      rope_pair(u[0], v[0], cs[0], sn[0], o1, o2);
      st1<T>(x, o1);
      st1<T>(x + half, o2);
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(256) rotate_slabs_kernel(const RotateHeads a) {
  const int n = a.H * a.dp, half = a.rot >> 1;
  const int c = blockIdx.y * 256 + threadIdx.x;
  const int64_t t = blockIdx.x;
  if (c >= n) return;
  const int d = c % a.dp;
  const bool hi = d >= a.d + half && d < a.d + a.rot;
  T* q = static_cast<T*>(a.q) + t * n + c;
  float u = 0.f;
  for (int s = 0; s < a.S; ++s) u += a.xp[t * n + c + s * a.slab];
  if (d < a.d || d >= a.d + a.rot) {
    st1<T>(q, u);
    return;
  }
  int64_t p = a.pos[t];
  p = p < 0 ? 0 : (p >= a.max_pos ? a.max_pos - 1 : p);
  const int i = d - a.d - (hi ? half : 0);
  float o = 0.f;
  for (int s = 0; s < a.S; ++s) o += a.xp[t * n + c + (hi ? -half : half) + s * a.slab];
  float o1, o2;
  rope_pair(hi ? o : u, hi ? u : o, a.cos_t[p * a.rot_ld + i], a.sin_t[p * a.rot_ld + i], o1, o2);
  st1<T>(q, hi ? o2 : o1);
}

int rotate_heads(const RotateHeads& a, int tokens, bool f32, hipStream_t stream) {
  if (tokens == 0) return 0;
  if (a.rot % 2 || a.d + a.rot > a.dp || a.H < 1) return -1;
  if (a.xp) {
    const dim3 grid(tokens, (a.H * a.dp + 255) / 256);
    if (f32) rotate_slabs_kernel<float><<<grid, 256, 0, stream>>>(a);
    else rotate_slabs_kernel<bf16_t><<<grid, 256, 0, stream>>>(a);
    OAMD_LAUNCH_CHECK();
    return 0;
  }
  if (a.rot == 0) return 0;
  const bool vec = (a.rot / 2) % 8 == 0 && a.d % 8 == 0 && a.dp % 8 == 0;
  const int64_t items = (int64_t)tokens * a.H * (a.rot / 2) / (vec ? 8 : 1);
  const int grid = (int)(items < 256 * 8192 ? (items + 255) / 256 : 8192);
  if (f32) {
    if (vec) rotate_rows_kernel<float, 8><<<grid, 256, 0, stream>>>(a, items);
    else rotate_rows_kernel<float, 1><<<grid, 256, 0, stream>>>(a, items);
  } else {
    if (vec) rotate_rows_kernel<bf16_t, 8><<<grid, 256, 0, stream>>>(a, items);
    else rotate_rows_kernel<bf16_t, 1><<<grid, 256, 0, stream>>>(a, items);
  }
  OAMD_LAUNCH_CHECK();
  return 0;
}

// Y[m][h][n] = sum_k X[m][h][k] W[h][n][k]; K % 8 == 0, N % 16 == 0. A workgroup is 16 columns of one head
// and 16 MT rows; its 4 waves take every fourth 32-deep step and are summed through LDS. Column
// groups past N copy the `nx` columns of X from column x0 on (zeros past them) to Y's columns N...
template <int MT>
__global__ void __launch_bounds__(256) head_gemm_kernel(const HeadGemm a) {
  __shared__ float red[4][MT][256];
  const int h = blockIdx.z, n0 = blockIdx.x * 16, m0 = blockIdx.y * 16 * MT;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, r = lane & 15, kq = lane >> 4;
  const bf16_t* X = a.X + (int64_t)h * a.xh;
  bf16_t* Y = a.Y + (int64_t)h * a.yh;
  if (n0 >= a.N) {
    for (int e = tid; e < 16 * 16 * MT; e += 256) {
      const int m = m0 + e / 16, c = n0 - a.N + e % 16;
      if (m < a.M) Y[(int64_t)m * a.ldy + a.N + c] = c < a.nx ? X[(int64_t)m * a.ldx + a.x0 + c] : (bf16_t)0;
    }
    return;
  }
  const bf16_t* W = a.W + ((int64_t)h * a.N + n0 + r) * a.K;
  f32x4 acc[MT];
#pragma unroll
  for (int j = 0; j < MT; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  for (int k = 32 * w + 8 * kq; k - 8 * kq < a.K; k += 128) {
    const bool ok = k < a.K;
    const u16x8 wf = ok ? *reinterpret_cast<const u16x8*>(W + k) : zero;
    u16x8 xf[MT];
#pragma unroll
    for (int j = 0; j < MT; ++j) {
      const int m = m0 + 16 * j + r;
      xf[j] = ok && m < a.M ? *reinterpret_cast<const u16x8*>(X + (int64_t)m * a.ldx + k) : zero;
    }
#pragma unroll
    for (int j = 0; j < MT; ++j)
      acc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, wf), __builtin_bit_cast(bf16x8, xf[j]),
                                                       acc[j], 0, 0, 0);
  }
  // lane l: row m = l & 15, columns 4 (l >> 4) + i
#pragma unroll
  for (int j = 0; j < MT; ++j) *reinterpret_cast<f32x4*>(&red[w][j][4 * lane]) = acc[j];
  __syncthreads();
  for (int e = tid; e < 64 * MT; e += 256) {
    const int j = e >> 6, l = e & 63, m = m0 + 16 * j + (l & 15);
    f32x4 v = *reinterpret_cast<const f32x4*>(&red[0][j][4 * l]);
#pragma unroll
    for (int ww = 1; ww < 4; ++ww) v += *reinterpret_cast<const f32x4*>(&red[ww][j][4 * l]);
    if (m < a.M)
      *reinterpret_cast<uint2*>(Y + (int64_t)m * a.ldy + n0 + 4 * (l >> 4)) = make_uint2(pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3]));
  }
}

int head_gemm(const HeadGemm& a, hipStream_t stream) {
  if (a.M == 0) return 0;
  if (a.K % 8 || a.N % 16 || a.pad % 16 || a.nx > a.pad || a.ldx % 8 || a.xh % 8 || a.ldy % 4 || a.yh % 4 || a.H < 1 || a.H > 65535) return -1;
  const int gx = (a.N + a.pad) / 16;
  if (a.M <= 16) head_gemm_kernel<1><<<dim3(gx, 1, a.H), 256, 0, stream>>>(a);
  else head_gemm_kernel<4><<<dim3(gx, (a.M + 63) / 64, a.H), 256, 0, stream>>>(a);
  OAMD_LAUNCH_CHECK();
  return 0;
}

}  // namespace oamd
