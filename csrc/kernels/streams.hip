// Hyper-connection step: a residual stream kept as S parallel fp32 copies per token.
//
// One launch finishes a sublayer and starts the next:
//   x'_t = sum_s mix[s][t] x_s + out[t] * y        (every stream from the old ones)
//   u    = sum_t in[t] x'_t                         (what the next sublayer reads)
//   h    = u / sqrt(mean(u^2) + eps) * w            (its pre-norm)
// so a token's S x width streams are read once and written once per sublayer, and the
// sublayer's output y never makes a separate pass: it comes as bf16 / fp32 rows, as the
// fp32 split-K slabs of the projection that made it, scaled by a per-token sigmoid gate,
// and / or as the rows of the experts a token was routed to.
// The first step (ids != nullptr) writes every stream from the scaled embedding row; the
// With post_w (one stream) y is itself divided by its root mean square and scaled before it joins. The
// last one (sum) normalises the plain sum of the streams and needs only the rows whose
// logits are wanted (rows). HBM-bound: 8 S bytes per feature per token plus y and h.
#include "common.h"
#include "kernels.h"

namespace oamd {

namespace {

__device__ __forceinline__ f32x4 ld4(const void* p, int64_t i, bool f32) {
  if (f32) return *reinterpret_cast<const f32x4*>(static_cast<const float*>(p) + i);
  const u16x4 v = *reinterpret_cast<const u16x4*>(static_cast<const bf16_t*>(p) + i);
  return f32x4{bf2f(v[0]), bf2f(v[1]), bf2f(v[2]), bf2f(v[3])};
}

}  // namespace

// One workgroup per row; thread t owns 4-feature vectors t, t + NT, ... (MAXV of them).
// S: compile-time bound of the stream count a.S. POST: y is normalised first (post_w).
template <int S, int NT, int MAXV, bool POST>
__global__ void __launch_bounds__(NT) stream_step_kernel(const StreamStep a) {
  __shared__ float scratch[NT / 64];
  __shared__ float coef[S * S + 2 * S];   // mix[from][to], out, in
  const int tid = threadIdx.x;
  const int64_t row = a.rows ? a.rows[blockIdx.x] : (int64_t)blockIdx.x;
  for (int i = tid; i < S * S + 2 * S; i += NT) {
    float v = 0.f;
    if (i < S * S) {
      const int f = i / S, t = i % S;
      if (a.mix && f < a.S && t < a.S) v = a.mix[f * a.S + t];
    } else if (i < S * S + S) {
      if (a.out && i - S * S < a.S) v = a.out[i - S * S];
    } else if (i - S * S - S < a.S) {
      v = a.sum ? 1.f : a.in[i - S * S - S];
    }
    coef[i] = v;
  }
  int64_t id = 0;
  if (a.ids) {
    id = a.ids[row];
    if (id < 0 || id >= a.vocab) id = 0;   // out-of-range ids never read past the table
  }
  float gate = 1.f;
  if (a.gate) gate = 1.f / (1.f + __expf(-a.gate[row]));
  __syncthreads();

  const int nv = a.ld >> 2;
  float* xr = a.x + row * (int64_t)a.S * a.ld;
  auto output = [&](int v) {   // 4 features of the sublayer's output
    f32x4 y = f32x4{0.f, 0.f, 0.f, 0.f};
    if (a.yp) {
      const float* p = a.yp + row * a.ld + 4 * v;
      int s0 = 0;
      if constexpr (MAXV == 1) {   // up to 8 slabs requested before the first add: one round trip
        f32x4 sl[8];
#pragma unroll
        for (int s = 0; s < 8; ++s)
          if (s < a.ys) sl[s] = *reinterpret_cast<const f32x4*>(p + s * a.y_slab);
#pragma unroll
        for (int s = 0; s < 8; ++s)
          if (s < a.ys) y += sl[s];
        s0 = 8;
      }
      for (int s = s0; s < a.ys; ++s) y += *reinterpret_cast<const f32x4*>(p + s * a.y_slab);
    } else if (a.y) {
      y = ld4(a.y, row * a.ld + 4 * v, a.f32);
    }
    if (a.gate) y *= gate;
    for (int k = 0; k < a.top; ++k) {
      const int64_t sl = row * a.top + k;
      const int64_t er = a.epos ? (int64_t)a.epos[sl] : sl;
      y += ld4(a.e, er * a.ld + 4 * v, a.f32);
    }
    return y;
  };
  f32x4 yn[POST ? MAXV : 1];
  if constexpr (POST) {
    float ys = 0.f;
#pragma unroll
    for (int i = 0; i < MAXV; ++i) {
      const int v = tid + i * NT;
      yn[i] = v < nv ? output(v) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < 4; ++j) ys += yn[i][j] * yn[i][j];
    }
    const float rs = 1.f / sqrtf(block_sum<NT>(ys, scratch) / static_cast<float>(a.width) + a.eps);
#pragma unroll
    for (int i = 0; i < MAXV; ++i) {
      const int v = tid + i * NT;
      if (v < nv) yn[i] *= rs * *reinterpret_cast<const f32x4*>(a.post_w + 4 * v);
    }
  }
  f32x4 u[MAXV];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int v = tid + i * NT;
    u[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (v < nv) {
      f32x4 nx[S];
      if (a.ids) {
        f32x4 e = ld4(a.table, id * a.ld + 4 * v, a.f32);
#pragma unroll
        for (int j = 0; j < 4; ++j) e[j] *= a.emb_scale;
#pragma unroll
        for (int t = 0; t < S; ++t) nx[t] = e;
      } else {
        f32x4 xo[S];
#pragma unroll
        for (int s = 0; s < S; ++s)
          xo[s] = s < a.S ? *reinterpret_cast<const f32x4*>(xr + (int64_t)s * a.ld + 4 * v) : f32x4{0.f, 0.f, 0.f, 0.f};
        f32x4 y;
        if constexpr (POST) y = yn[i];
        else y = output(v);
#pragma unroll
        for (int t = 0; t < S; ++t) {
          f32x4 n = y * coef[S * S + t];
#pragma unroll
          for (int s = 0; s < S; ++s) n += xo[s] * coef[s * S + t];
          nx[t] = n;
        }
      }
      if (a.write_x) {
#pragma unroll
        for (int t = 0; t < S; ++t)
          if (t < a.S) *reinterpret_cast<f32x4*>(xr + (int64_t)t * a.ld + 4 * v) = nx[t];
      }
#pragma unroll
      for (int t = 0; t < S; ++t) u[i] += nx[t] * coef[S * S + S + t];
#pragma unroll
      for (int j = 0; j < 4; ++j) ss += u[i][j] * u[i][j];
    }
  }
  const float tot = block_sum<NT>(ss, scratch);
  const float rs = rsqrtf(tot / static_cast<float>(a.width) + a.eps);
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int v = tid + i * NT;
    if (v < nv) {
      const f32x4 w = *reinterpret_cast<const f32x4*>(a.w + 4 * v);
      const f32x4 o = u[i] * rs * w;
      const int64_t at = blockIdx.x * (int64_t)a.ld + 4 * v;
      if (a.f32) *reinterpret_cast<f32x4*>(static_cast<float*>(a.h) + at) = o;
      else *reinterpret_cast<uint2*>(static_cast<bf16_t*>(a.h) + at) = make_uint2(pack_bf2(o[0], o[1]), pack_bf2(o[2], o[3]));
    }
  }
}

template <int S, bool POST = false>
static void launch_streams(const StreamStep& a, int n, hipStream_t stream) {
  const int nv = a.ld / 4;
  if constexpr (S <= 4) {
    // few rows (decode): a vector per thread, so a row's loads all leave in one round trip
    if (n <= 512 && nv > 256) {
      if (nv <= 512) stream_step_kernel<S, 512, 1, POST><<<n, 512, 0, stream>>>(a);
      else if (nv <= 1024) stream_step_kernel<S, 1024, 1, POST><<<n, 1024, 0, stream>>>(a);
      else if (nv <= 2048) stream_step_kernel<S, 1024, 2, POST><<<n, 1024, 0, stream>>>(a);
      else stream_step_kernel<S, 1024, 4, POST><<<n, 1024, 0, stream>>>(a);
      return;
    }
  }
  if (nv <= 64) stream_step_kernel<S, 64, 1, POST><<<n, 64, 0, stream>>>(a);
  else if (nv <= 256) stream_step_kernel<S, 256, 1, POST><<<n, 256, 0, stream>>>(a);
  else if (nv <= 1024) stream_step_kernel<S, 256, 4, POST><<<n, 256, 0, stream>>>(a);
  else if (nv <= 2048) stream_step_kernel<S, 256, 8, POST><<<n, 256, 0, stream>>>(a);
  else stream_step_kernel<S, 256, 16, POST><<<n, 256, 0, stream>>>(a);
}

int stream_step(const StreamStep& a, int n_rows, hipStream_t stream) {
  if (n_rows == 0) return 0;
  if (a.S < 1 || a.S > 8 || a.ld % 8 != 0 || a.ld > 16384 || a.width < 1 || a.width > a.ld) return -1;
  if (a.post_w && a.S != 1) return -2;
  if (a.post_w) launch_streams<1, true>(a, n_rows, stream);
  else if (a.S == 1) launch_streams<1>(a, n_rows, stream);
  else if (a.S == 2) launch_streams<2>(a, n_rows, stream);
  else if (a.S <= 4) launch_streams<4>(a, n_rows, stream);
  else launch_streams<8>(a, n_rows, stream);
  OAMD_LAUNCH_CHECK();
  return 0;
}

}  // namespace oamd
