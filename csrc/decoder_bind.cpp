// Python bindings of the general decoder ops (operator_amd._C): hyper-connection streams,
// QKV head preparation, short-convolution heads, latent attention, attention with any head size, routed
// experts, fp32 products.
//
// As in bindings.cpp, every shape a kernel's grid or addressing relies on is checked on the
// host before the launch.
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>
#include <ATen/hip/impl/HIPGuardImplMasqueradingAsCUDA.h>
#include <ATen/hip/impl/HIPStreamMasqueradingAsCUDA.h>

#include "kernels/kernels.h"

namespace {

using oamd::bf16_t;
using OptT = c10::optional<at::Tensor>;

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStreamMasqueradingAsCUDA().stream(); }

#define RC(call)                                                         \
  do {                                                                   \
    int rc__ = (call);                                                   \
    TORCH_CHECK(rc__ == 0, "kernel launch failed: " #call " rc=", rc__); \
  } while (0)

// sliding windows: 0 = none
int window_of(int64_t w) { return w > 0 && w < oamd::kNoWindow ? (int)w : oamd::kNoWindow; }

// contiguous GPU tensor of `dt` with exactly (or at least) n elements
void need(const at::Tensor& t, at::ScalarType dt, int64_t n, const char* what, bool at_least = false) {
  TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == dt, what, ": contiguous GPU tensor of ", dt,
              " expected, got ", t.scalar_type());
  TORCH_CHECK(at_least ? t.numel() >= n : t.numel() == n, what, ": ", n, " elements expected, got ", t.numel());
}

template <typename T>
T* p(const at::Tensor& t) { return reinterpret_cast<T*>(t.data_ptr()); }
template <typename T>
T* op(const OptT& t) { return t.has_value() ? reinterpret_cast<T*>(t->data_ptr()) : nullptr; }
void* vp(const OptT& t) { return t.has_value() ? t->data_ptr() : nullptr; }

bool elem_f32(const at::Tensor& t, const char* what) {
  TORCH_CHECK(t.scalar_type() == at::kFloat || t.scalar_type() == at::kBFloat16, what, ": bf16 or fp32 expected");
  return t.scalar_type() == at::kFloat;
}

// x [T, S, ld] fp32 streams; h [rows, ld] output. ids: first step. y / slabs / e: see StreamStep.
void stream_step(at::Tensor& x, at::Tensor& h, int64_t width, const at::Tensor& w, double eps, const OptT& in,
                 const OptT& ids, const OptT& table, double emb_scale, const OptT& y, const OptT& slabs,
                 int64_t splits, const OptT& gate, const OptT& e, const OptT& epos, int64_t top, const OptT& mix,
                 const OptT& out, const OptT& rows, bool write_x, const OptT& post_w) {
  TORCH_CHECK(x.dim() == 3 && h.dim() == 2 && h.size(1) == x.size(2), "stream_step: x [T, S, ld], h [rows, ld]");
  const int64_t T = x.size(0), S = x.size(1), ld = x.size(2), n = h.size(0);
  need(x, at::kFloat, T * S * ld, "x");
  const bool f32 = elem_f32(h, "h");
  const auto dt = h.scalar_type();
  need(h, dt, n * ld, "h");
  need(w, at::kFloat, ld, "norm weight");
  TORCH_CHECK(width >= 1 && width <= ld, "stream_step: width");
  oamd::StreamStep a{};
  a.x = p<float>(x);
  a.S = (int)S;
  a.width = (int)width;
  a.ld = (int)ld;
  if (ids.has_value()) {
    TORCH_CHECK(table.has_value() && table->dim() == 2 && table->size(1) == ld, "stream_step: table [vocab, ld]");
    need(*ids, at::kLong, T, "ids");
    need(*table, dt, table->numel(), "table");
    a.ids = p<int64_t>(*ids);
    a.table = table->data_ptr();
    a.vocab = table->size(0);
    a.emb_scale = (float)emb_scale;
  } else {
    TORCH_CHECK(mix.has_value() && out.has_value(), "stream_step: mix and out of the finished sublayer");
    need(*mix, at::kFloat, S * S, "mix");
    need(*out, at::kFloat, S, "out");
    a.mix = p<float>(*mix);
    a.out = p<float>(*out);
    if (slabs.has_value()) {
      TORCH_CHECK(splits >= 1, "stream_step: splits");
      need(*slabs, at::kFloat, splits * T * ld, "slabs", true);
      a.yp = p<float>(*slabs);
      a.ys = (int)splits;
      a.y_slab = T * ld;
    } else if (y.has_value()) {
      need(*y, dt, T * ld, "y");
      a.y = y->data_ptr();
    }
    if (gate.has_value()) {
      need(*gate, at::kFloat, T, "gate");
      a.gate = p<float>(*gate);
    }
    if (top > 0) {
      TORCH_CHECK(e.has_value() && e->dim() == 2 && e->size(1) == ld, "stream_step: e [rows, ld]");
      need(*e, dt, e->numel(), "e");
      if (epos.has_value()) need(*epos, at::kInt, T * top, "epos");   // values: moe_sort rows, all below e's row count
      else TORCH_CHECK(e->size(0) >= T * top, "stream_step: e rows");
      a.e = e->data_ptr();
      a.epos = op<int>(epos);
      a.top = (int)top;
    }
  }
  if (in.has_value()) {
    need(*in, at::kFloat, S, "in");
    a.in = p<float>(*in);
  }
  a.sum = !in.has_value();
  if (post_w.has_value()) {
    TORCH_CHECK(S == 1 && !ids.has_value(), "stream_step: the output norm belongs to a finished sublayer of one stream");
    need(*post_w, at::kFloat, ld, "post_w");
    a.post_w = p<float>(*post_w);
  }
  a.w = p<float>(w);
  a.h = h.data_ptr();
  a.eps = (float)eps;
  a.f32 = f32;
  a.write_x = write_x;
  if (rows.has_value()) {
    need(*rows, at::kLong, n, "rows");
    TORCH_CHECK(a.sum && !ids.has_value() && !write_x, "stream_step: rows only in a last step that keeps the streams");
    a.rows = p<int64_t>(*rows);
  } else {
    TORCH_CHECK(n == T, "stream_step: h rows");
  }
  const c10::hip::HIPGuardMasqueradingAsCUDA g(x.device());
  RC(oamd::stream_step(a, (int)n, cur_stream()));
}

void qkv_heads(const at::Tensor& qkv, const OptT& slabs, int64_t splits, const OptT& bias, const at::Tensor& pos,
               const OptT& cos_t, const OptT& sin_t, int64_t rot_pairs, int64_t Hq, int64_t Hkv, int64_t dk,
               bool norm, double eps, const OptT& v_first, const OptT& lam, at::Tensor& q_out, const OptT& k_out,
               const OptT& v_out, const OptT& k_cache, const OptT& v_cache, const OptT& slots, int64_t dvp,
               int64_t ncol) {
  const bool f32 = elem_f32(q_out, "q_out");
  const auto dt = q_out.scalar_type();
  const int64_t T = pos.numel();
  TORCH_CHECK(q_out.dim() == 3 && q_out.size(0) == T && q_out.size(1) == Hq, "qkv_heads: q_out [T, Hq, dkp]");
  const int64_t dkp = q_out.size(2);
  need(q_out, dt, T * Hq * dkp, "q_out");
  need(pos, at::kLong, T, "pos");
  TORCH_CHECK(Hq >= 1 && Hkv >= 1 && dk >= 1 && dk <= dkp && ncol >= (Hq + Hkv) * dkp + Hkv * dvp && ncol % 8 == 0 &&
                  dkp % 8 == 0 && dvp % 8 == 0 && 2 * rot_pairs <= dk,
              "qkv_heads: head sizes");
  oamd::QkvHeads a{};
  if (slabs.has_value()) {
    need(*slabs, at::kFloat, splits * T * ncol, "slabs", true);
    a.xp = p<float>(*slabs);
    a.S = (int)splits;
    a.slab = T * ncol;
  } else {
    need(qkv, dt, T * ncol, "qkv");
    a.row = qkv.data_ptr();
    a.S = 1;
  }
  a.ncol = (int)ncol;
  if (bias.has_value()) {
    need(*bias, at::kFloat, ncol, "bias");
    a.bias = p<float>(*bias);
  }
  a.pos = p<int64_t>(pos);
  if (rot_pairs > 0) {
    TORCH_CHECK(cos_t.has_value() && sin_t.has_value() && cos_t->dim() == 2 && cos_t->sizes() == sin_t->sizes() &&
                    cos_t->size(1) % 4 == 0 && cos_t->size(1) >= rot_pairs && cos_t->size(0) >= 1,
                "qkv_heads: cos / sin [max_pos, >= rot_pairs, % 4]");
    need(*cos_t, at::kFloat, cos_t->numel(), "cos");
    need(*sin_t, at::kFloat, sin_t->numel(), "sin");
    a.cos_t = p<float>(*cos_t);
    a.sin_t = p<float>(*sin_t);
    a.rot_ld = (int)cos_t->size(1);
    a.max_pos = cos_t->size(0);
  }
  a.rot_pairs = (int)rot_pairs;
  a.Hq = (int)Hq; a.Hkv = (int)Hkv; a.dk = (int)dk; a.dkp = (int)dkp; a.dvp = (int)dvp;
  a.norm = norm;
  a.eps = (float)eps;
  if (v_first.has_value()) {
    TORCH_CHECK(lam.has_value(), "qkv_heads: lam");
    need(*v_first, dt, T * Hkv * dvp, "v_first");
    need(*lam, at::kFloat, 1, "lam");
    a.v_first = v_first->data_ptr();
    a.lam = p<float>(*lam);
  }
  a.q_out = q_out.data_ptr();
  if (k_out.has_value()) need(*k_out, dt, T * Hkv * dkp, "k_out");
  if (v_out.has_value()) need(*v_out, dt, T * Hkv * dvp, "v_out");
  a.k_out = vp(k_out);
  a.v_out = vp(v_out);
  if (k_cache.has_value()) {
    TORCH_CHECK(v_cache.has_value() && slots.has_value(), "qkv_heads: k_cache needs v_cache and slots");
    TORCH_CHECK(k_cache->dim() == 4 && v_cache->dim() == 4 && k_cache->size(1) == Hkv && v_cache->size(1) == Hkv &&
                    k_cache->size(0) == v_cache->size(0) && k_cache->size(2) == v_cache->size(2) &&
                    k_cache->size(3) == dkp && v_cache->size(3) == dvp,
                "qkv_heads: cache [pages, Hkv, page, size]");
    need(*k_cache, dt, k_cache->numel(), "k_cache");
    need(*v_cache, dt, v_cache->numel(), "v_cache");
    need(*slots, at::kLong, T, "slots");
    a.k_cache = k_cache->data_ptr();
    a.v_cache = v_cache->data_ptr();
    a.slots = p<int64_t>(*slots);
    const int64_t P = k_cache->size(2);
    TORCH_CHECK(P >= 1 && (P & (P - 1)) == 0, "qkv_heads: pages of a power of two tokens");
    while ((1 << a.log2_page) < P) ++a.log2_page;
  }
  const c10::hip::HIPGuardMasqueradingAsCUDA g(pos.device());
  RC(oamd::qkv_heads(a, (int)T, f32, cur_stream()));
}

// o: [T, o_ld] rows, head h at column h * dvp
void attn_gd_prefill(const at::Tensor& q, const at::Tensor& k, const at::Tensor& v, at::Tensor& o,
                     const at::Tensor& cu, const OptT& work_seq, const OptT& work_q0, double scale, const OptT& pk,
                     const OptT& pv, const OptT& seq_pfx, int64_t window, const OptT& gate) {
  TORCH_CHECK(q.dim() == 3 && k.dim() == 3 && v.dim() == 3 && o.dim() == 2, "attn_gd_prefill: q, k, v [T, H, d], o [T, ld]");
  const int64_t T = q.size(0), Hq = q.size(1), dkp = q.size(2), Hkv = k.size(1), dvp = v.size(2);
  const bool f32 = elem_f32(q, "q");
  const auto dt = q.scalar_type();
  need(q, dt, T * Hq * dkp, "q");
  need(k, dt, T * Hkv * dkp, "k");
  need(v, dt, T * Hkv * dvp, "v");
  need(o, dt, T * o.size(1), "o");
  TORCH_CHECK(v.size(1) == Hkv && Hkv >= 1 && Hq % Hkv == 0 && o.size(1) >= Hq * dvp, "attn_gd_prefill: heads");
  need(cu, at::kInt, cu.numel(), "cu_seqlens");
  const int64_t seqs = cu.numel() - 1;
  TORCH_CHECK(seqs >= 1, "attn_gd_prefill: cu_seqlens");
  const int win = window_of(window);
  if (gate.has_value()) need(*gate, at::kFloat, T * Hq, "gate");
  if (pk.has_value()) {
    TORCH_CHECK(pv.has_value() && seq_pfx.has_value() && pk->dim() == 3 && pk->size(0) == pv->size(0), "attn_gd_prefill: prefix");
    need(*pk, dt, pk->size(0) * Hkv * dkp, "pk");
    need(*pv, dt, pk->size(0) * Hkv * dvp, "pv");
    need(*seq_pfx, at::kInt, seqs, "seq_pfx");
  }
  const c10::hip::HIPGuardMasqueradingAsCUDA g(q.device());
  if (f32) {
    oamd::AttnF32 a{};
    a.q = p<float>(q); a.k = p<float>(k); a.v = p<float>(v); a.o = p<float>(o);
    a.o_ld = (int)o.size(1);
    a.cu_seqlens = p<int>(cu);
    a.num_seqs = (int)seqs;
    a.Hkv = (int)Hkv; a.dkp = (int)dkp; a.dvp = (int)dvp;
    a.k_ld = dkp; a.v_ld = dvp;
    a.window = win; a.gate = op<float>(gate);
    a.scale = (float)scale;
    a.pk = op<float>(pk); a.pv = op<float>(pv); a.seq_pfx = op<int>(seq_pfx);
    RC(oamd::attn_f32(a, (int)T, (int)Hq, false, cur_stream()));
    return;
  }
  TORCH_CHECK(work_seq.has_value() && work_q0.has_value(), "attn_gd_prefill: work list");
  need(*work_seq, at::kInt, work_seq->numel(), "work_seq");
  need(*work_q0, at::kInt, work_seq->numel(), "work_q0");
  oamd::AttnPrefill a{};
  a.q = p<bf16_t>(q); a.k = p<bf16_t>(k); a.v = p<bf16_t>(v); a.o = p<bf16_t>(o);
  a.o_ld = (int)o.size(1);
  TORCH_CHECK(a.o_ld % 4 == 0, "attn_gd_prefill: o rows");
  a.cu_seqlens = p<int>(cu); a.work_seq = p<int>(*work_seq); a.work_q0 = p<int>(*work_q0);
  a.Hkv = (int)Hkv;
  a.G = (int)(Hq / Hkv);
  a.gc = a.G % 4 == 0 ? 4 : a.G % 3 == 0 ? 3 : a.G % 2 == 0 ? 2 : 1;
  a.dkp = (int)dkp; a.dvp = (int)dvp;
  a.scale_log2 = (float)(scale * 1.4426950408889634);
  a.pk = op<bf16_t>(pk); a.pv = op<bf16_t>(pv); a.seq_pfx = op<int>(seq_pfx);
  a.window = win; a.gate = op<float>(gate);
  RC(oamd::attn_gd_prefill(a, (int)work_seq->numel(), cur_stream()));
}

void attn_gd_decode(const at::Tensor& q, const at::Tensor& k_cache, const at::Tensor& v_cache, const at::Tensor& bt,
                    const at::Tensor& lens, at::Tensor& o, const OptT& o_part, const OptT& ml_part,
                    int64_t num_splits, double scale, int64_t window, const OptT& gate) {
  TORCH_CHECK(q.dim() == 3 && k_cache.dim() == 4 && v_cache.dim() == 4 && bt.dim() == 2 && o.dim() == 2,
              "attn_gd_decode: q [B, Hq, d], cache [pages, Hkv, page, d], bt [B, max_pages], o [B, ld]");
  const int64_t B = q.size(0), Hq = q.size(1), dkp = q.size(2), Hkv = k_cache.size(1), P = k_cache.size(2),
                dvp = v_cache.size(3);
  const bool f32 = elem_f32(q, "q");
  const auto dt = q.scalar_type();
  need(q, dt, B * Hq * dkp, "q");
  need(k_cache, dt, k_cache.numel(), "k_cache");
  need(v_cache, dt, v_cache.numel(), "v_cache");
  need(bt, at::kInt, B * bt.size(1), "block_tables");
  need(lens, at::kInt, B, "seq_lens");
  need(o, dt, B * o.size(1), "o");
  TORCH_CHECK(k_cache.size(3) == dkp && v_cache.size(1) == Hkv && v_cache.size(2) == P && v_cache.size(0) == k_cache.size(0) &&
                  Hq % Hkv == 0 && o.size(1) >= Hq * dvp && P >= 16 && (P & (P - 1)) == 0 && num_splits >= 1,
              "attn_gd_decode: shapes");
  if (gate.has_value()) need(*gate, at::kFloat, B * Hq, "gate");
  const int win = window_of(window);
  const c10::hip::HIPGuardMasqueradingAsCUDA g(q.device());
  if (f32) {
    oamd::AttnF32 a{};
    a.q = p<float>(q); a.k = p<float>(k_cache); a.v = p<float>(v_cache); a.o = p<float>(o);
    a.o_ld = (int)o.size(1);
    a.block_tables = p<int>(bt); a.seq_lens = p<int>(lens);
    a.Hkv = (int)Hkv; a.dkp = (int)dkp; a.dvp = (int)dvp;
    a.page_size = (int)P; a.max_pages = (int)bt.size(1);
    a.k_ld = dkp; a.v_ld = dvp;
    a.window = win; a.gate = op<float>(gate);
    a.scale = (float)scale;
    RC(oamd::attn_f32(a, (int)B, (int)Hq, true, cur_stream()));
    return;
  }
  oamd::AttnDecode a{};
  a.q = p<bf16_t>(q); a.k_cache = p<bf16_t>(k_cache); a.v_cache = p<bf16_t>(v_cache);
  a.block_tables = p<int>(bt); a.seq_lens = p<int>(lens);
  a.out = p<bf16_t>(o);
  a.o_ld = (int)o.size(1);
  if (num_splits > 1) {
    TORCH_CHECK(o_part.has_value() && ml_part.has_value(), "attn_gd_decode: workspace");
    need(*o_part, at::kFloat, B * Hq * num_splits * dvp, "o_part", true);
    need(*ml_part, at::kFloat, B * Hq * num_splits * 2, "ml_part", true);
    a.o_part = p<float>(*o_part); a.ml_part = p<float>(*ml_part);
  }
  a.Hkv = (int)Hkv; a.G = (int)(Hq / Hkv); a.dkp = (int)dkp; a.dvp = (int)dvp;
  a.page_size = (int)P; a.max_pages = (int)bt.size(1); a.num_splits = (int)num_splits;
  int lg = 0;
  while ((1 << lg) < P) ++lg;
  a.log2_page = lg;
  a.scale_log2 = (float)(scale * 1.4426950408889634);
  a.window = win;
  a.gate = op<float>(gate);
  RC(oamd::attn_gd_decode(a, (int)B, cur_stream()));
}

// q [B, H, ck]; cache [pages, 1, P, ck] token rows whose first rp columns are the values; o [B, H * rp]
void attn_latent_decode(const at::Tensor& q, const at::Tensor& cache, const at::Tensor& bt, const at::Tensor& lens,
                        at::Tensor& o, int64_t rp, const OptT& o_part, const OptT& ml_part, int64_t num_splits, double scale,
                        const OptT& gate) {
  TORCH_CHECK(q.dim() == 3 && cache.dim() == 4 && bt.dim() == 2 && o.dim() == 2 && cache.size(1) == 1 && cache.size(3) == q.size(2),
              "attn_latent_decode: q [B, H, ck], cache [pages, 1, page, ck], bt [B, max_pages], o [B, H rp]");
  const int64_t B = q.size(0), H = q.size(1), ck = q.size(2), P = cache.size(2);
  const bool f32 = elem_f32(q, "q");
  const auto dt = q.scalar_type();
  need(q, dt, B * H * ck, "q");
  need(cache, dt, cache.numel(), "cache");
  need(bt, at::kInt, B * bt.size(1), "block_tables");
  need(lens, at::kInt, B, "seq_lens");
  need(o, dt, B * H * rp, "o");
  TORCH_CHECK(P >= 16 && (P & (P - 1)) == 0 && num_splits >= 1 && rp >= 16 && rp % 16 == 0 && rp <= ck, "attn_latent_decode: shapes");
  if (gate.has_value()) need(*gate, at::kFloat, B * H, "gate");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(q.device());
  if (f32) {
    oamd::AttnF32 a{};
    a.q = p<float>(q); a.k = a.v = p<float>(cache); a.o = p<float>(o);
    a.o_ld = (int)(H * rp);
    a.block_tables = p<int>(bt); a.seq_lens = p<int>(lens);
    a.Hkv = 1; a.dkp = (int)ck; a.dvp = (int)rp; a.k_ld = a.v_ld = ck;
    a.page_size = (int)P; a.max_pages = (int)bt.size(1);
    a.scale = (float)scale;
    a.window = oamd::kNoWindow; a.gate = op<float>(gate);
    RC(oamd::attn_f32(a, (int)B, (int)H, true, cur_stream()));
    return;
  }
  oamd::AttnDecode a{};
  a.q = p<bf16_t>(q); a.k_cache = p<bf16_t>(cache);
  a.block_tables = p<int>(bt); a.seq_lens = p<int>(lens);
  a.out = p<bf16_t>(o);
  a.o_ld = (int)(H * rp);
  if (num_splits > 1) {
    TORCH_CHECK(o_part.has_value() && ml_part.has_value(), "attn_latent_decode: workspace");
    need(*o_part, at::kFloat, B * H * num_splits * rp, "o_part", true);
    need(*ml_part, at::kFloat, B * H * num_splits * 2, "ml_part", true);
    a.o_part = p<float>(*o_part); a.ml_part = p<float>(*ml_part);
  }
  a.Hkv = 1; a.G = (int)H; a.dkp = (int)ck; a.dvp = (int)rp;
  a.page_size = (int)P; a.max_pages = (int)bt.size(1); a.num_splits = (int)num_splits;
  while ((1 << a.log2_page) < P) ++a.log2_page;
  a.scale_log2 = (float)(scale * 1.4426950408889634);
  a.window = oamd::kNoWindow;
  a.gate = op<float>(gate);
  RC(oamd::attn_latent_decode(a, (int)B, (int)rp, cur_stream()));
}

// packed projection [T, ncol] as rows of dtype dt, or `splits` fp32 slabs
template <typename A>
void set_rows(A& a, const at::Tensor& x, const OptT& slabs, int64_t splits, int64_t T, int64_t ncol, at::ScalarType dt) {
  if (slabs.has_value()) {
    TORCH_CHECK(splits >= 1, "splits");
    need(*slabs, at::kFloat, splits * T * ncol, "slabs", true);
    a.xp = p<float>(*slabs);
    a.S = (int)splits;
    a.slab = T * ncol;
  } else {
    need(x, dt, T * ncol, "projection rows");
    a.row = x.data_ptr();
    a.S = 1;
  }
}

int page_log2(int64_t P) {
  TORCH_CHECK(P >= 16 && (P & (P - 1)) == 0, "pages of a power of two tokens, at least 16");
  int lg = 0;
  while ((1 << lg) < P) ++lg;
  return lg;
}

template <typename A>
void set_tables(A& a, const at::Tensor& cos_t, const at::Tensor& sin_t, int64_t rot) {
  TORCH_CHECK(cos_t.dim() == 2 && cos_t.sizes() == sin_t.sizes() && cos_t.size(1) >= rot / 2 && cos_t.size(0) >= 1, "cos / sin [max_pos, >= rot / 2]");
  need(cos_t, at::kFloat, cos_t.numel(), "cos");
  need(sin_t, at::kFloat, sin_t.numel(), "sin");
  a.cos_t = p<float>(cos_t);
  a.sin_t = p<float>(sin_t);
  a.rot_ld = (int)cos_t.size(1);
  a.max_pos = cos_t.size(0);
}

void conv_heads(const at::Tensor& x, const OptT& slabs, int64_t splits, const at::Tensor& conv, const at::Tensor& qw,
                const at::Tensor& kw, const at::Tensor& pos, int64_t dk, double eps, at::Tensor& q_out, const OptT& k_out,
                const OptT& v_out, at::Tensor& k_cache, at::Tensor& v_cache, const at::Tensor& slots, const OptT& tails,
                at::Tensor& gate, int64_t ncol, const OptT& cu, const OptT& prev_page, const OptT& bt) {
  const bool f32 = elem_f32(q_out, "q_out");
  const auto dt = q_out.scalar_type();
  TORCH_CHECK(q_out.dim() == 3 && k_cache.dim() == 4 && v_cache.dim() == 4 && conv.dim() == 2, "conv_heads: q_out [T, Hq, dkp], cache [pages, Hkv, page, d], conv [taps, C]");
  const int64_t T = pos.numel(), Hq = q_out.size(1), dkp = q_out.size(2), Hkv = k_cache.size(1), dvp = v_cache.size(3);
  const int64_t taps = conv.size(0), C = (Hq + Hkv) * dkp, pages = k_cache.size(0), P = k_cache.size(2);
  need(pos, at::kLong, T, "pos");
  need(q_out, dt, T * Hq * dkp, "q_out");
  need(conv, dt, taps * C, "conv");
  need(qw, dt, dkp, "q norm weight");
  need(kw, dt, dkp, "k norm weight");
  need(gate, at::kFloat, T * Hq, "gate");
  need(slots, at::kLong, T, "slots");
  need(k_cache, dt, pages * Hkv * P * dkp, "k_cache");
  need(v_cache, dt, pages * Hkv * P * dvp, "v_cache");
  TORCH_CHECK(dk >= 1 && dk <= dkp && dvp >= dkp && ncol >= C + Hq && ncol % 8 == 0 && P >= taps - 1, "conv_heads: sizes");
  oamd::ConvHeads a{};
  a.T = (int)T;
  set_rows(a, x, slabs, splits, T, ncol, dt);
  a.ncol = (int)ncol;
  a.taps = (int)taps;
  a.conv = conv.data_ptr(); a.qw = qw.data_ptr(); a.kw = kw.data_ptr();
  a.pos = p<int64_t>(pos);
  a.Hq = (int)Hq; a.Hkv = (int)Hkv; a.dk = (int)dk; a.dkp = (int)dkp; a.dvp = (int)dvp;
  a.eps = (float)eps;
  TORCH_CHECK(cu.has_value() != bt.has_value(), "conv_heads: sequence starts (prefill) or block tables (decode)");
  if (cu.has_value()) {
    a.num_seqs = (int)cu->numel() - 1;
    TORCH_CHECK(a.num_seqs >= 1, "conv_heads: cu_seqlens");
    need(*cu, at::kInt, a.num_seqs + 1, "cu_seqlens");
    a.cu_seqlens = p<int>(*cu);
    if (prev_page.has_value()) {
      need(*prev_page, at::kInt, a.num_seqs, "prev_page");
      a.prev_page = p<int>(*prev_page);
    }
  } else {
    TORCH_CHECK(bt->dim() == 2 && bt->size(0) == T, "conv_heads: block tables [T, max_pages]");
    need(*bt, at::kInt, bt->numel(), "block_tables");
    a.block_tables = p<int>(*bt);
    a.max_pages = (int)bt->size(1);
  }
  a.pages = pages;
  if (taps > 1) {
    TORCH_CHECK(tails.has_value(), "conv_heads: tails");
    need(*tails, dt, pages * (taps - 1) * C, "tails");
    a.tails = tails->data_ptr();
  }
  if (k_out.has_value()) need(*k_out, dt, T * Hkv * dkp, "k_out");
  if (v_out.has_value()) need(*v_out, dt, T * Hkv * dvp, "v_out");
  a.q_out = q_out.data_ptr();
  a.k_out = vp(k_out);
  a.v_out = vp(v_out);
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  a.slots = p<int64_t>(slots);
  a.log2_page = page_log2(P);
  a.gate = p<float>(gate);
  const c10::hip::HIPGuardMasqueradingAsCUDA g(pos.device());
  RC(oamd::conv_heads(a, f32, cur_stream()));
}

// lat / cache absent: the layer reads another layer's latent rows
void latent_rows(const at::Tensor& x, const OptT& slabs, int64_t splits, int64_t ncol, int64_t q_rank, int64_t kv_rank, int64_t rp,
                 int64_t rot, int64_t rotp, const at::Tensor& qw, const OptT& cw, double eps, const at::Tensor& pos,
                 const at::Tensor& cos_t, const at::Tensor& sin_t, at::Tensor& cq, const OptT& lat, const OptT& cache,
                 const OptT& slots, at::Tensor& gate) {
  const bool f32 = elem_f32(cq, "cq");
  const auto dt = cq.scalar_type();
  TORCH_CHECK(cq.dim() == 2 && gate.dim() == 2, "latent_rows: cq [T, qp], gate [T, H]");
  const int64_t T = pos.numel(), qp = cq.size(1), H = gate.size(1);
  need(pos, at::kLong, T, "pos");
  need(cq, dt, T * qp, "cq");
  need(gate, at::kFloat, T * H, "gate");
  need(qw, at::kFloat, qp, "query latent norm weight");
  TORCH_CHECK(q_rank >= 1 && q_rank <= qp && ncol % 8 == 0, "latent_rows: query latent");
  oamd::LatentRows a{};
  set_rows(a, x, slabs, splits, T, ncol, dt);
  a.ncol = (int)ncol;
  a.q_rank = (int)q_rank; a.qp = (int)qp; a.H = (int)H;
  a.qw = p<float>(qw);
  a.eps = (float)eps;
  a.pos = p<int64_t>(pos);
  a.cq = cq.data_ptr();
  a.gate = p<float>(gate);
  int64_t used = qp + H;
  if (lat.has_value()) {
    TORCH_CHECK(cw.has_value() && cache.has_value() && slots.has_value() && lat->dim() == 2 && cache->dim() == 4 && cache->size(1) == 1 &&
                    cache->size(3) == lat->size(1), "latent_rows: lat [T, ck], cache [pages, 1, page, ck]");
    const int64_t ck = lat->size(1);
    need(*lat, dt, T * ck, "lat");
    need(*cache, dt, cache->numel(), "cache");
    need(*slots, at::kLong, T, "slots");
    need(*cw, at::kFloat, rp, "latent norm weight");
    TORCH_CHECK(kv_rank >= 1 && kv_rank <= rp && rot >= 0 && rot % 2 == 0 && rot <= rotp && rp + rot <= ck, "latent_rows: sizes");
    page_log2(cache->size(2));
    set_tables(a, cos_t, sin_t, rot);
    a.kv_rank = (int)kv_rank; a.rp = (int)rp; a.rot = (int)rot; a.rotp = (int)rotp; a.ck = (int)ck;
    a.cw = p<float>(*cw);
    a.lat = lat->data_ptr();
    a.cache = cache->data_ptr();
    a.slots = p<int64_t>(*slots);
    used += rp + rotp;
  }
  TORCH_CHECK(ncol >= used, "latent_rows: columns");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(pos.device());
  RC(oamd::latent_rows(a, (int)T, f32, cur_stream()));
}

void rotate_heads(at::Tensor& q, const OptT& slabs, int64_t splits, int64_t d, int64_t rot, const at::Tensor& pos,
                  const at::Tensor& cos_t, const at::Tensor& sin_t) {
  TORCH_CHECK(q.dim() == 3 && q.size(0) == pos.numel(), "rotate_heads: q [T, H, dp]");
  const bool f32 = elem_f32(q, "q");
  need(q, q.scalar_type(), q.numel(), "q");
  need(pos, at::kLong, q.size(0), "pos");
  TORCH_CHECK(rot >= 0 && rot % 2 == 0 && d >= 0 && d + rot <= q.size(2), "rotate_heads: sizes");
  oamd::RotateHeads a{};
  a.q = q.data_ptr();
  if (slabs.has_value()) {
    need(*slabs, at::kFloat, splits * q.numel(), "slabs", true);
    a.xp = p<float>(*slabs);
    a.S = (int)splits;
    a.slab = q.numel();
  }
  a.pos = p<int64_t>(pos);
  set_tables(a, cos_t, sin_t, rot);
  a.H = (int)q.size(1); a.dp = (int)q.size(2); a.d = (int)d; a.rot = (int)rot;
  const c10::hip::HIPGuardMasqueradingAsCUDA g(q.device());
  RC(oamd::rotate_heads(a, (int)q.size(0), f32, cur_stream()));
}

// x [M, H, xd], w [H, N, K <= xd], y [M, H, >= N]: y[m, h, :N] = x[m, h, :K] w[h]^T; columns past N: x[m, h, x0 : x0 + nx],
// then zeros. y [M, >= H N]: rows with head h at column h N.
void head_gemm(const at::Tensor& x, const at::Tensor& w, at::Tensor& y, int64_t x0, int64_t nx) {
  TORCH_CHECK(x.dim() == 3 && w.dim() == 3 && x.size(0) == y.size(0) && x.size(1) == w.size(0) &&
                  (y.dim() == 3 ? y.size(1) == w.size(0) : y.dim() == 2 && y.size(1) >= w.size(0) * w.size(1) && nx == 0),
              "head_gemm: x [M, H, xd], w [H, N, K], y [M, H, yd]");
  const int64_t M = x.size(0), H = x.size(1), xd = x.size(2), N = w.size(1), K = w.size(2), yd = y.dim() == 3 ? y.size(2) : N;
  const int64_t ldy = y.dim() == 3 ? H * yd : y.size(1);
  const bool f32 = elem_f32(x, "x");
  const auto dt = x.scalar_type();
  need(x, dt, M * H * xd, "x");
  need(w, dt, w.numel(), "w");
  need(y, dt, M * ldy, "y");
  TORCH_CHECK(K <= xd && N <= yd && K % 16 == 0 && N % 16 == 0 && xd % 8 == 0 && yd % 16 == 0 && x0 >= 0 && nx >= 0 && x0 + nx <= xd &&
                  nx <= yd - N, "head_gemm: sizes");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(x.device());
  if (f32) {
    RC(oamd::head_gemm_f32(p<float>(x), p<float>(w), p<float>(y), (int)M, (int)N, (int)K, (int)H, H * xd, xd, ldy, yd, cur_stream()));
    return;
  }
  oamd::HeadGemm a{};
  a.X = p<bf16_t>(x); a.W = p<bf16_t>(w); a.Y = p<bf16_t>(y);
  a.M = (int)M; a.N = (int)N; a.K = (int)K; a.H = (int)H;
  a.ldx = H * xd; a.xh = xd; a.ldy = ldy; a.yh = yd;
  a.pad = (int)(yd - N); a.x0 = (int)x0; a.nx = (int)nx;
  RC(oamd::head_gemm(a, cur_stream()));
}

void gemm_f32(const at::Tensor& x, const at::Tensor& w, at::Tensor& y, int64_t silu_gu, const OptT& gtab, const OptT& rscale) {
  TORCH_CHECK(x.dim() == 2 && y.dim() == 2, "gemm_f32: x [M, K], y [M, N]");
  const int64_t M = x.size(0), K = x.size(1), N = w.size(-2);
  need(x, at::kFloat, M * K, "x");
  need(w, at::kFloat, w.numel(), "w");
  need(y, at::kFloat, M * (silu_gu ? N / 2 : N), "y");
  TORCH_CHECK(w.size(-1) == K && y.size(0) == M && K % 16 == 0 && (!silu_gu || N % 128 == 0), "gemm_f32: shapes");
  if (gtab.has_value()) {
    TORCH_CHECK(w.dim() == 3 && M % 64 == 0, "gemm_f32: expert rows come in 64-row tiles, w [experts, N, K]");
    need(*gtab, at::kInt, 1 + M / 64, "gtab", true);
  } else {
    TORCH_CHECK(w.dim() == 2, "gemm_f32: w [N, K]");
  }
  if (rscale.has_value()) need(*rscale, at::kFloat, M, "rscale");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(x.device());
  RC(oamd::gemm_f32(p<float>(x), p<float>(w), p<float>(y), (int)M, (int)N, (int)K, (int)y.size(1), (int)silu_gu,
                    op<int>(gtab), op<float>(rscale), cur_stream()));
}

void moe_route(const at::Tensor& h, const at::Tensor& wr, int64_t E, at::Tensor& ids, at::Tensor& weights,
               const OptT& gate, const OptT& logits) {
  TORCH_CHECK(h.dim() == 2 && wr.dim() == 2 && ids.dim() == 2 && wr.size(1) == h.size(1), "moe_route: h [T, K], wr [rows, K]");
  const int64_t T = h.size(0), K = h.size(1), rows = wr.size(0), top = ids.size(1);
  need(h, at::kBFloat16, T * K, "h");
  need(wr, at::kBFloat16, rows * K, "wr");
  need(ids, at::kInt, T * top, "ids");
  need(weights, at::kFloat, T * top, "weights");
  if (gate.has_value()) need(*gate, at::kFloat, T, "gate");
  if (logits.has_value()) need(*logits, at::kFloat, T * E, "logits");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(h.device());
  RC(oamd::moe_route(p<bf16_t>(h), p<bf16_t>(wr), (int)T, (int)K, (int)E, (int)rows, (int)top, p<int>(ids),
                     p<float>(weights), op<float>(gate), op<float>(logits), cur_stream()));
}

void moe_topk(const at::Tensor& logits, int64_t E, at::Tensor& ids, at::Tensor& weights, const OptT& gate) {
  TORCH_CHECK(logits.dim() == 2 && ids.dim() == 2, "moe_topk: logits [T, ld], ids [T, top]");
  const int64_t T = logits.size(0), top = ids.size(1);
  need(logits, at::kFloat, logits.numel(), "logits");
  need(ids, at::kInt, T * top, "ids");
  need(weights, at::kFloat, T * top, "weights");
  if (gate.has_value()) need(*gate, at::kFloat, T, "gate");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(logits.device());
  RC(oamd::moe_topk(p<float>(logits), (int)logits.size(1), (int)T, (int)E, (int)top, p<int>(ids), p<float>(weights),
                    op<float>(gate), cur_stream()));
}

// ids must come from moe_route / moe_topk (every value inside [0, E))
void moe_sort(const at::Tensor& ids, const at::Tensor& weights, int64_t E, int64_t bm, at::Tensor& pos, at::Tensor& src,
              at::Tensor& rscale, at::Tensor& gtab) {
  TORCH_CHECK(ids.dim() == 2, "moe_sort: ids [T, top]");
  const int64_t slots = ids.numel(), rows = src.numel();
  need(ids, at::kInt, slots, "ids");
  need(weights, at::kFloat, slots, "weights");
  need(pos, at::kInt, slots, "pos");
  need(src, at::kInt, rows, "src");
  need(rscale, at::kFloat, rows, "rscale");
  TORCH_CHECK(bm > 0 && rows % bm == 0, "moe_sort: rows");
  need(gtab, at::kInt, 1 + rows / bm, "gtab", true);
  const c10::hip::HIPGuardMasqueradingAsCUDA g(ids.device());
  RC(oamd::moe_sort(p<int>(ids), p<float>(weights), (int)slots, (int)ids.size(1), (int)E, (int)bm, (int)rows,
                    p<int>(pos), p<int>(src), p<float>(rscale), p<int>(gtab), cur_stream()));
}

void moe_gather(const at::Tensor& h, const at::Tensor& src, const at::Tensor& gtab, int64_t bm, at::Tensor& xp) {
  TORCH_CHECK(h.dim() == 2 && xp.dim() == 2 && h.size(1) == xp.size(1) && h.scalar_type() == xp.scalar_type(), "moe_gather: shapes");
  need(h, h.scalar_type(), h.numel(), "h");
  need(xp, h.scalar_type(), xp.numel(), "xp");
  need(src, at::kInt, xp.size(0), "src");
  need(gtab, at::kInt, 1 + xp.size(0) / bm, "gtab", true);
  const c10::hip::HIPGuardMasqueradingAsCUDA g(h.device());
  RC(oamd::moe_gather(h.data_ptr(), p<int>(src), p<int>(gtab), (int)bm, (int)xp.size(0), xp.data_ptr(),
                      (int)(h.size(1) * h.element_size()), cur_stream()));
}

void moe_gemm_skinny(const at::Tensor& x, const at::Tensor& w, at::Tensor& y, const at::Tensor& ids,
                     const at::Tensor& weights, int64_t div, bool silu_gu) {
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && y.dim() == 2 && w.size(2) == x.size(1), "moe_gemm_skinny: x [.., K], w [E, N, K]");
  const int64_t slots = ids.numel(), E = w.size(0), N = w.size(1), K = w.size(2);
  need(x, at::kBFloat16, x.numel(), "x");
  need(w, at::kBFloat16, w.numel(), "w");
  need(ids, at::kInt, slots, "ids");
  need(weights, at::kFloat, slots, "weights");
  need(y, at::kBFloat16, slots * (silu_gu ? N / 2 : N), "y");
  TORCH_CHECK(div >= 1 && x.size(0) * div >= slots && E <= 65535, "moe_gemm_skinny: rows");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(x.device());
  RC(oamd::moe_gemm_skinny(p<bf16_t>(x), p<bf16_t>(w), p<bf16_t>(y), p<int>(ids), p<float>(weights), (int)slots,
                           (int)div, (int)E, (int)N, (int)K, silu_gu, cur_stream()));
}

// rows: moe_sort's, in tiles of bm; src given: x [T, K] is gathered by it (values < T)
void moe_gemm_rows(const at::Tensor& x, const at::Tensor& w, at::Tensor& y, int64_t bm, const at::Tensor& gtab,
                   const OptT& src, const OptT& rscale, bool silu_gu) {
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && y.dim() == 2 && w.size(2) == x.size(1), "moe_gemm_rows: x [.., K], w [E, N, K]");
  const int64_t M = y.size(0), N = w.size(1), K = w.size(2);
  need(x, at::kBFloat16, x.numel(), "x");
  need(w, at::kBFloat16, w.numel(), "w");
  need(y, at::kBFloat16, M * (silu_gu ? N / 2 : N), "y");
  TORCH_CHECK((bm == 64 || bm == 128) && M % bm == 0 && (src.has_value() || x.size(0) == M) && x.size(0) >= 1, "moe_gemm_rows: rows");
  need(gtab, at::kInt, 1 + M / bm, "gtab", true);
  if (src.has_value()) need(*src, at::kInt, M, "src");
  if (rscale.has_value()) need(*rscale, at::kFloat, M, "rscale");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(x.device());
  RC(oamd::moe_gemm_rows(p<bf16_t>(x), p<bf16_t>(w), p<bf16_t>(y), (int)M, (int)N, (int)K, (int)bm, silu_gu, p<int>(gtab),
                         op<int>(src), op<float>(rscale), cur_stream()));
}

void splitk_silu(const at::Tensor& slabs, at::Tensor& y, int64_t splits, int64_t glu) {
  TORCH_CHECK(y.dim() == 2 && splits >= 1, "splitk_silu: y [M, N / 2]");
  need(y, at::kBFloat16, y.numel(), "y");
  need(slabs, at::kFloat, splits * y.numel() * 2, "slabs", true);
  const c10::hip::HIPGuardMasqueradingAsCUDA g(y.device());
  RC(oamd::splitk_silu(p<float>(slabs), p<bf16_t>(y), (int)y.size(0), (int)y.size(1) * 2, (int)splits, (int)glu, cur_stream()));
}

void moe_gemm_tile(const at::Tensor& x, const at::Tensor& w, at::Tensor& y, const at::Tensor& gtab, const OptT& rscale,
                   bool silu_gu) {
  TORCH_CHECK(x.dim() == 2 && w.dim() == 3 && y.dim() == 2 && w.size(2) == x.size(1), "moe_gemm_tile: x [rows, K], w [E, N, K]");
  const int64_t M = x.size(0), N = w.size(1), K = w.size(2);
  need(x, at::kBFloat16, M * K, "x");
  need(w, at::kBFloat16, w.numel(), "w");
  need(y, at::kBFloat16, M * (silu_gu ? N / 2 : N), "y");
  TORCH_CHECK(M % 256 == 0 && K <= (1 << 21), "moe_gemm_tile: 256-row tiles");
  need(gtab, at::kInt, 1 + M / 256, "gtab", true);
  if (rscale.has_value()) need(*rscale, at::kFloat, M, "rscale");
  const c10::hip::HIPGuardMasqueradingAsCUDA g(x.device());
  RC(oamd::moe_gemm_tile(p<bf16_t>(x), p<bf16_t>(w), p<bf16_t>(y), (int)M, (int)N, (int)K, silu_gu, p<int>(gtab),
                         op<float>(rscale), cur_stream()));
}

}  // namespace

void register_decoder_bindings(pybind11::module_& m) {
  namespace py = pybind11;
  const py::none no;
  m.def("stream_step", &stream_step, py::arg("x"), py::arg("h"), py::arg("width"), py::arg("w"), py::arg("eps"),
        py::arg("in_") = no, py::arg("ids") = no, py::arg("table") = no, py::arg("emb_scale") = 1.0, py::arg("y") = no,
        py::arg("slabs") = no, py::arg("splits") = 1, py::arg("gate") = no, py::arg("e") = no, py::arg("epos") = no,
        py::arg("top") = 0, py::arg("mix") = no, py::arg("out") = no, py::arg("rows") = no, py::arg("write_x") = true, py::arg("post_w") = no);
  m.def("qkv_heads", &qkv_heads, py::arg("qkv"), py::arg("slabs"), py::arg("splits"), py::arg("bias"), py::arg("pos"),
        py::arg("cos"), py::arg("sin"), py::arg("rot_pairs"), py::arg("Hq"), py::arg("Hkv"), py::arg("dk"),
        py::arg("norm"), py::arg("eps"), py::arg("v_first"), py::arg("lam"), py::arg("q_out"), py::arg("k_out"),
        py::arg("v_out"), py::arg("k_cache"), py::arg("v_cache"), py::arg("slots"), py::arg("dvp"), py::arg("ncol"));
  m.def("attn_gd_prefill", &attn_gd_prefill, py::arg("q"), py::arg("k"), py::arg("v"), py::arg("o"), py::arg("cu"),
        py::arg("work_seq") = no, py::arg("work_q0") = no, py::arg("scale") = 1.0, py::arg("pk") = no,
        py::arg("pv") = no, py::arg("seq_pfx") = no, py::arg("window") = 0, py::arg("gate") = no);
  m.def("attn_gd_decode", &attn_gd_decode, py::arg("q"), py::arg("k_cache"), py::arg("v_cache"), py::arg("bt"),
        py::arg("lens"), py::arg("o"), py::arg("o_part") = no, py::arg("ml_part") = no, py::arg("num_splits") = 1,
        py::arg("scale") = 1.0, py::arg("window") = 0, py::arg("gate") = no);
  m.def("attn_latent_decode", &attn_latent_decode, py::arg("q"), py::arg("cache"), py::arg("bt"), py::arg("lens"), py::arg("o"),
        py::arg("rp"), py::arg("o_part") = no, py::arg("ml_part") = no, py::arg("num_splits") = 1, py::arg("scale") = 1.0,
        py::arg("gate") = no);
  m.def("conv_heads", &conv_heads, py::arg("x"), py::arg("slabs"), py::arg("splits"), py::arg("conv"), py::arg("qw"), py::arg("kw"),
        py::arg("pos"), py::arg("dk"), py::arg("eps"), py::arg("q_out"), py::arg("k_out"), py::arg("v_out"), py::arg("k_cache"),
        py::arg("v_cache"), py::arg("slots"), py::arg("tails"), py::arg("gate"), py::arg("ncol"), py::arg("cu") = no,
        py::arg("prev_page") = no, py::arg("bt") = no);
  m.def("latent_rows", &latent_rows, py::arg("x"), py::arg("slabs"), py::arg("splits"), py::arg("ncol"), py::arg("q_rank"),
        py::arg("kv_rank"), py::arg("rp"), py::arg("rot"), py::arg("rotp"), py::arg("qw"), py::arg("cw"), py::arg("eps"),
        py::arg("pos"), py::arg("cos"), py::arg("sin"), py::arg("cq"), py::arg("lat"), py::arg("cache"), py::arg("slots"),
        py::arg("gate"));
  m.def("rotate_heads", &rotate_heads, py::arg("q"), py::arg("slabs"), py::arg("splits"), py::arg("d"), py::arg("rot"),
        py::arg("pos"), py::arg("cos"), py::arg("sin"));
  m.def("head_gemm", &head_gemm, py::arg("x"), py::arg("w"), py::arg("y"), py::arg("x0") = 0, py::arg("nx") = 0);
  m.def("gemm_f32", &gemm_f32, py::arg("x"), py::arg("w"), py::arg("y"), py::arg("silu_gu") = 0,
        py::arg("gtab") = no, py::arg("rscale") = no);
  m.def("moe_route", &moe_route, py::arg("h"), py::arg("wr"), py::arg("E"), py::arg("ids"), py::arg("weights"),
        py::arg("gate") = no, py::arg("logits") = no);
  m.def("moe_topk", &moe_topk, py::arg("logits"), py::arg("E"), py::arg("ids"), py::arg("weights"), py::arg("gate") = no);
  m.def("moe_sort", &moe_sort);
  m.def("moe_gather", &moe_gather);
  m.def("moe_gemm_skinny", &moe_gemm_skinny, py::arg("x"), py::arg("w"), py::arg("y"), py::arg("ids"),
        py::arg("weights"), py::arg("div"), py::arg("silu_gu"));
  m.def("moe_gemm_rows", &moe_gemm_rows, py::arg("x"), py::arg("w"), py::arg("y"), py::arg("bm"), py::arg("gtab"),
        py::arg("src") = no, py::arg("rscale") = no, py::arg("silu_gu") = false);
  m.def("splitk_silu", &splitk_silu, py::arg("slabs"), py::arg("y"), py::arg("splits"), py::arg("glu") = 1);
  m.def("moe_gemm_tile", &moe_gemm_tile, py::arg("x"), py::arg("w"), py::arg("y"), py::arg("gtab"),
        py::arg("rscale") = no, py::arg("silu_gu") = false);
}
