// pybind11 layer of the mixer-stack serving kernels: every shape, dtype and
// range that a kernel relies on is checked here, on the host.
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

#include <cmath>

#include "lm.h"

namespace {

using torch::Tensor;
using OptTensor = c10::optional<Tensor>;

hipStream_t cur_stream() { return c10::hip::getCurrentHIPStream().stream(); }

void launched() {
  const hipError_t e = hipGetLastError();
  TORCH_CHECK(e == hipSuccess, "HIP error: ", hipGetErrorString(e));
}

bool is_f32(const Tensor& t) {
  TORCH_CHECK(t.scalar_type() == torch::kBFloat16 || t.scalar_type() == torch::kFloat32,
              "bfloat16 or float32 expected");
  return t.scalar_type() == torch::kFloat32;
}

void dense(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be on the GPU");
  TORCH_CHECK(t.is_contiguous(), name, " must be contiguous");
}

void shaped(const Tensor& t, torch::IntArrayRef shape, c10::ScalarType type,
            const char* name) {
  dense(t, name);
  TORCH_CHECK(t.sizes() == shape, name, ": shape ", t.sizes(), ", expected ", shape);
  TORCH_CHECK(t.scalar_type() == type, name, ": wrong dtype");
}

const void* opt_vec(const OptTensor& t, long n, c10::ScalarType type,
                    const char* name) {
  if (!t.has_value()) return nullptr;
  shaped(*t, {n}, type, name);
  return t->data_ptr();
}

const int* ints(const Tensor& t, long n, const char* name) {
  dense(t, name);
  TORCH_CHECK(t.scalar_type() == torch::kInt32 && t.numel() >= n, name,
              ": int32 with at least ", n, " entries expected");
  return t.data_ptr<int>();
}

void width_ok(long W) {
  TORCH_CHECK(W >= 1 && W <= (W % 4 == 0 ? 16384 : 4096), "unsupported width ", W);
}

LmNorm norm_of(const OptTensor& w, const OptTensor& b, const OptTensor& alpha,
               bool rms, long W, c10::ScalarType type, const char* name) {
  LmNorm n{};
  n.one = w.has_value() && w->dim() == 0;      // one number for all columns
  if (n.one) {
    shaped(*w, {}, type, name);
    n.w = w->data_ptr();
  } else {
    n.w = opt_vec(w, W, type, name);
  }
  n.b = opt_vec(b, W, type, name);
  n.rms = rms;
  if (alpha.has_value()) {
    TORCH_CHECK(n.w && n.b && alpha->is_cuda() && alpha->numel() == 1 &&
                alpha->scalar_type() == type, name, ": alpha");
    n.alpha = alpha->data_ptr();
  }
  return n;
}

const long* token_ids(const Tensor& t, long T) {
  dense(t, "tokens");
  TORCH_CHECK(t.scalar_type() == torch::kInt64 && t.numel() == T,
              "tokens: ", T, " int64 expected");
  return t.data_ptr<int64_t>();
}

float* stream_x(const Tensor& x) {
  dense(x, "x");
  TORCH_CHECK(x.dim() == 2 && x.scalar_type() == torch::kFloat32,
              "the stream is a float32 matrix");
  width_ok(x.size(1));
  return x.data_ptr<float>();
}

// y (T, W), or y (T, n, W) with float weights (T, n)
LmSum sum_of(const OptTensor& y, const OptTensor& weights, long T, long W,
             c10::ScalarType type) {
  LmSum s{};
  if (!y.has_value()) return s;
  s.y = y->data_ptr();
  if (weights.has_value()) {
    TORCH_CHECK(weights->dim() == 2, "weights of the parts");
    s.n = (int)weights->size(1);
    shaped(*weights, {T, s.n}, torch::kFloat32, "weights of the parts");
    shaped(*y, {T, s.n, W}, type, "parts of a sublayer's output");
    s.w = weights->data_ptr<float>();
  } else {
    shaped(*y, {T, W}, type, "sublayer output");
  }
  return s;
}

// tokens (T,) -> x (T, W) float stream, returns its norm h (T, W); ptab:
// learned positions to add at pos
std::vector<Tensor> embed_norm(Tensor tokens, Tensor embed, OptTensor pos,
                               OptTensor ptab, OptTensor w, OptTensor b,
                               OptTensor alpha, bool rms, double eps) {
  dense(embed, "embed");
  const bool f32 = is_f32(embed);
  const long T = tokens.numel(), V = embed.size(0), W = embed.size(1);
  const long* tp = token_ids(tokens, T);
  width_ok(W);
  auto x = torch::empty({T, W}, embed.options().dtype(torch::kFloat32));
  auto h = torch::empty({T, W}, embed.options());
  const int* pp = nullptr;
  const void* tab = nullptr;
  long np = 0;
  if (ptab.has_value()) {
    TORCH_CHECK(pos.has_value() && ptab->dim() == 2, "positions");
    pp = ints(*pos, T, "positions");
    np = ptab->size(0);
    shaped(*ptab, {np, W}, embed.scalar_type(), "learned positions");
    tab = ptab->data_ptr();
  }
  lm_embed_norm(tp, embed.data_ptr(), pp, tab, (int)np, x.data_ptr<float>(),
                norm_of(w, b, alpha, rms, W, embed.scalar_type(), "norm"),
                h.data_ptr(), (int)T, (int)W, V, (float)eps, f32, cur_stream());
  launched();
  return {x, h};
}

// x += mult * N(y; post); returns N(x; next) of `rows` (or all rows)
Tensor residual_norm(Tensor x, OptTensor y, OptTensor weights, OptTensor pw,
                     OptTensor pb, OptTensor pa, bool p_rms, double mult,
                     OptTensor nw, OptTensor nb, OptTensor na, bool n_rms,
                     OptTensor rows, double eps, bool store_x) {
  TORCH_CHECK(nw.has_value() || y.has_value(), "a norm or a sublayer output");
  const Tensor& like = nw.has_value() ? *nw : *y;
  const bool f32 = is_f32(like);
  const auto ty = like.scalar_type();
  float* xp = stream_x(x);
  const long T = x.size(0), W = x.size(1);
  const LmSum sum = sum_of(y, weights, T, W, ty);
  long n = T;
  const int* rp = nullptr;
  if (rows.has_value()) {
    n = rows->numel();
    rp = ints(*rows, n, "rows");
    TORCH_CHECK(!store_x, "a row subset leaves the stream alone");
  }
  auto h = torch::empty({n, W}, like.options());
  lm_residual_norm(xp, sum,
                   norm_of(pw, pb, pa, p_rms, W, ty, "post norm"), (float)mult,
                   norm_of(nw, nb, na, n_rms, W, ty, "norm"), h.data_ptr(), rp,
                   (int)n, (int)W, (float)eps, store_x, f32, cur_stream());
  launched();
  return h;
}

// x += mult * N(y; post); returns rows [x | embed[token]]
Tensor residual_concat(Tensor x, OptTensor y, OptTensor weights, OptTensor pw,
                       OptTensor pb, OptTensor pa, bool p_rms, double mult,
                       Tensor tokens, Tensor embed, double eps) {
  dense(embed, "embed");
  const bool f32 = is_f32(embed);
  const auto ty = embed.scalar_type();
  float* xp = stream_x(x);
  const long T = x.size(0), W = x.size(1);
  TORCH_CHECK(embed.dim() == 2 && embed.size(1) == W, "embedding width");
  const long* tp = token_ids(tokens, T);
  auto h = torch::empty({T, 2 * W}, embed.options());
  lm_residual_concat(xp, sum_of(y, weights, T, W, ty),
                     norm_of(pw, pb, pa, p_rms, W, ty, "post norm"), (float)mult, tp,
                     embed.data_ptr(), h.data_ptr(), (int)T, (int)W,
                     embed.size(0), (float)eps, f32, cur_stream());
  launched();
  return h;
}

// x <- y + step; returns N(x; next)
Tensor replace_norm(Tensor x, Tensor y, Tensor step, OptTensor nw, OptTensor nb,
                    OptTensor na, bool n_rms, double eps) {
  const bool f32 = is_f32(step);
  const auto ty = step.scalar_type();
  float* xp = stream_x(x);
  const long T = x.size(0), W = x.size(1);
  const bool yf = y.scalar_type() == torch::kFloat32;
  shaped(y, {T, W}, yf ? torch::kFloat32 : ty, "projection");
  shaped(step, {W}, ty, "step");
  auto h = torch::empty({T, W}, step.options());
  lm_replace_norm(xp, y.data_ptr(), yf, step.data_ptr(),
                  norm_of(nw, nb, na, n_rms, W, ty, "norm"), h.data_ptr(), (int)T,
                  (int)W, (float)eps, f32, cur_stream());
  launched();
  return h;
}

// a gated activation of rows [gate | up]
Tensor gated(const Tensor& x, int act, double limit, double alpha, double shift) {
  dense(x, "x");
  TORCH_CHECK(x.dim() == 2 && x.size(1) % 2 == 0, "rows [gate | up] expected");
  const long n = x.size(1) / 2;
  auto y = torch::empty({x.size(0), n}, x.options());
  lm_gated_act(x.data_ptr(), y.data_ptr(), x.size(0), (int)n, act, (float)limit,
               (float)alpha, (float)shift, is_f32(x), cur_stream());
  launched();
  return y;
}

Tensor geglu_tanh(Tensor x) { return gated(x, LM_GELU_TANH, 0, 0, 0); }

Tensor clamped_glu(Tensor x, double limit, double alpha, double shift) {
  return gated(x, LM_CLAMPED, limit, alpha, shift);
}

Tensor softcap(Tensor x, double cap) {
  dense(x, "x");
  TORCH_CHECK(cap > 0, "cap");
  auto y = torch::empty(x.sizes(), x.options().dtype(torch::kFloat32));
  lm_softcap(x.data_ptr(), y.data_ptr<float>(), x.numel(), (float)cap,
             is_f32(x), cur_stream());
  launched();
  return y;
}

Tensor grouped_rms(Tensor y, Tensor w, long parts, double eps) {
  dense(y, "y");
  TORCH_CHECK(y.dim() == 2 && parts >= 1 && y.size(1) % parts == 0, "norm parts");
  shaped(w, {y.size(1)}, y.scalar_type(), "norm weight");
  TORCH_CHECK(y.size(0) * parts < (1L << 31), "too many rows");
  auto out = torch::empty_like(y);
  lm_grouped_rms(y.data_ptr(), w.data_ptr(), nullptr, 0, out.data_ptr(),
                 y.size(0), (int)parts, (int)(y.size(1) / parts), (float)eps,
                 is_f32(y), cur_stream());
  launched();
  return out;
}

// RMS norm of whole rows, times the sigmoid of p's columns from `col` on
Tensor gated_rms(Tensor y, Tensor w, Tensor p, long col, double eps) {
  dense(y, "y"); dense(p, "p");
  const long n = y.size(1);
  shaped(w, {n}, y.scalar_type(), "norm weight");
  TORCH_CHECK(y.dim() == 2 && p.dim() == 2 && p.size(0) == y.size(0) &&
              p.scalar_type() == y.scalar_type() && col >= 0 &&
              col + n <= p.size(1), "gates");
  TORCH_CHECK(y.size(0) < (1L << 31), "too many rows");
  auto out = torch::empty_like(y);
  lm_grouped_rms(y.data_ptr(), w.data_ptr(),
                 (const char*)p.data_ptr() + col * p.element_size(), p.size(1),
                 out.data_ptr(), y.size(0), 1, (int)n, (float)eps, is_f32(y),
                 cur_stream());
  launched();
  return out;
}

Tensor gelu_erf(Tensor x) {
  dense(x, "x");
  auto y = torch::empty_like(x);
  lm_gelu_erf(x.data_ptr(), y.data_ptr(), x.numel(), is_f32(x), cur_stream());
  launched();
  return y;
}

AttnArgs attn_args(const Tensor& qkv, const Tensor& kc, const Tensor& vc,
                   const Tensor& table, const OptTensor& qw, const OptTensor& kw,
                   const OptTensor& sink, const OptTensor& slopes, long heads,
                   long size, double scale, double eps) {
  const auto ty = qkv.scalar_type();
  dense(qkv, "qkv"); dense(kc, "key cache"); dense(vc, "value cache");
  dense(table, "page table");
  TORCH_CHECK(kc.dim() == 4 && vc.dim() == 4 && table.dim() == 2, "cache ranks");
  AttnArgs a{};
  a.H = (int)heads;
  a.G = (int)kc.size(1);
  a.dim = (int)kc.size(3);
  a.vdim = (int)vc.size(3);
  TORCH_CHECK(a.G >= 1 && a.H >= 1 && a.H % a.G == 0, "kv heads must divide heads");
  TORCH_CHECK(a.dim >= 1 && a.dim <= 256 && a.vdim >= 1 && a.vdim <= 256,
              "head sizes 1..256 are supported");
  TORCH_CHECK(kc.size(2) == LM_PAGE && vc.size(2) == LM_PAGE, "page length");
  shaped(vc, {kc.size(0), a.G, LM_PAGE, a.vdim}, ty, "value cache");
  TORCH_CHECK(kc.scalar_type() == ty, "key cache dtype");
  a.ld = (long)(a.H + a.G) * a.dim + (long)a.G * a.vdim;
  TORCH_CHECK(qkv.dim() == 2 && qkv.size(1) == a.ld, "qkv row length");
  TORCH_CHECK(size >= 0, "chunk size");
  a.qkv = qkv.data_ptr(); a.kc = kc.data_ptr(); a.vc = vc.data_ptr();
  a.qw = opt_vec(qw, a.dim, ty, "q norm");
  a.kw = opt_vec(kw, a.dim, ty, "k norm");
  a.sink = opt_vec(sink, a.H, ty, "sink");
  a.has_sink = a.sink != nullptr;
  a.slopes = (const float*)opt_vec(slopes, a.H, torch::kFloat32, "slopes");
  a.table = ints(table, 1, "page table");
  a.max_pages = (int)table.size(1);
  a.size = (int)size; a.scale = (float)scale; a.eps = (float)eps;
  a.out_scale = 1.f;
  return a;
}

// Rows [0, n_dec) of a.qkv are single new tokens, the rest prompt portions
// described by `tiles`; returns (T, heads * vdim), or fills a.out if it is set.
Tensor attend(AttnArgs& a, const Tensor& qkv, const Tensor& pos,
              const Tensor& slot, const Tensor& tiles, long n_dec,
              long max_len) {
  const bool f32 = is_f32(qkv);
  const long T = qkv.size(0);
  TORCH_CHECK(n_dec >= 0 && n_dec <= T, "decode rows");
  const int* pp = ints(pos, T, "positions");
  const int* sp = ints(slot, T, "slots");
  const long nt = tiles.numel() / 4;
  const int4* tp = (const int4*)ints(tiles, 4 * nt, "tiles");
  Tensor out;
  if (!a.out) {
    out = torch::empty({T, (long)a.H * a.vdim}, qkv.options());
    a.out = out.data_ptr();
    a.ldo = out.size(1);
  }
  auto st = cur_stream();
  if (n_dec > 0) {
    TORCH_CHECK(n_dec <= 65535, "too many decode rows");
    // enough blocks to fill the chip, none with fewer than ~128 keys;
    // the merge takes at most 64 splits
    const long hg = a.H / a.G;
    const long hc = !f32 && lm_attn_decode_tied_mfma(a) ? 16 : hg <= 2 ? hg : 4;
    const long blocks = n_dec * a.G * ((hg + hc - 1) / hc);
    const long keys = a.size > 0 ? std::min<long>(a.size + a.keep, max_len) : max_len;
    long ns = std::min((512 + blocks - 1) / blocks, (keys + 127) / 128);
    ns = std::max<long>(1, std::min<long>(ns, 64));
    Tensor ws;
    if (ns > 1)
      ws = torch::empty({n_dec * a.H * ns * (a.vdim + 2)},
                        qkv.options().dtype(torch::kFloat32));
    lm_attn_decode(a, pp, sp, (int)n_dec, (int)ns,
                   ns > 1 ? ws.data_ptr<float>() : nullptr, f32, st);
  }
  if (nt > 0) {
    TORCH_CHECK(a.H <= 65535, "too many heads");
    lm_attn_prep(a, pp, sp, (int)n_dec, (int)(T - n_dec), f32, st);
    lm_attn_prefill(a, tp, (int)nt, f32, st);
  }
  launched();
  return out;
}

// rows [q | k | v]
Tensor paged_attention(Tensor qkv, Tensor kc, Tensor vc, Tensor table,
                       Tensor pos, Tensor slot, Tensor tiles, long n_dec,
                       OptTensor qw, OptTensor kw, OptTensor sink,
                       OptTensor slopes, long heads, long size, double scale,
                       double eps, long max_len) {
  AttnArgs a = attn_args(qkv, kc, vc, table, qw, kw, sink, slopes, heads, size,
                         scale, eps);
  return attend(a, qkv, pos, slot, tiles, n_dec, max_len);
}

// columns [col, ...) of x: [q | k | v | gate]; result into columns
// [out_col, ...) of out
void window_attention(Tensor x, long col, Tensor out, long out_col, Tensor kc,
                      Tensor vc, Tensor table, Tensor pos, Tensor slot,
                      Tensor tiles, long n_dec, Tensor bias, double softcap,
                      long heads, long size, long keep, double scale,
                      double out_scale, double eps, long max_len) {
  const auto ty = x.scalar_type();
  is_f32(x);
  dense(x, "rows"); dense(out, "out"); dense(kc, "key cache");
  dense(vc, "value cache"); dense(table, "page table"); dense(bias, "bias");
  TORCH_CHECK(x.dim() == 2 && out.dim() == 2 && kc.dim() == 4 && vc.dim() == 4 &&
              table.dim() == 2 && bias.dim() == 2, "ranks");
  AttnArgs a{};
  a.H = (int)heads;
  a.G = (int)kc.size(1);
  a.dim = (int)kc.size(3);
  a.vdim = (int)vc.size(3);
  TORCH_CHECK(a.G >= 1 && a.H >= 1 && a.H % a.G == 0, "kv heads must divide heads");
  TORCH_CHECK(a.dim >= 1 && a.dim <= 256 && a.vdim >= 1 && a.vdim <= 256,
              "head sizes 1..256 are supported");
  TORCH_CHECK(kc.size(2) == LM_PAGE && kc.scalar_type() == ty, "key cache");
  shaped(vc, {kc.size(0), a.G, LM_PAGE, a.vdim}, ty, "value cache");
  a.ld = x.size(1);
  const long qk = (long)(a.H + a.G) * a.dim, g0 = qk + (long)a.G * a.vdim;
  TORCH_CHECK(col >= 0 && col % 8 == 0 && a.ld % 8 == 0 &&
              col + g0 + (long)a.H * a.vdim <= a.ld, "row length ", a.ld);
  a.ldo = out.size(1);
  TORCH_CHECK(out.size(0) == x.size(0) && out.scalar_type() == ty &&
              out_col >= 0 && out_col + (long)a.H * a.vdim <= a.ldo, "out");
  shaped(bias, {a.H, bias.size(1)}, torch::kFloat32, "bias");
  TORCH_CHECK(bias.size(1) >= 1 && size >= 0 && keep >= 0 && softcap >= 0,
              "window, bias, soft cap");
  const size_t es = x.element_size();
  a.qkv = (char*)x.data_ptr() + col * es;
  a.gate = (const char*)a.qkv + g0 * es;
  a.out = (char*)out.data_ptr() + out_col * es;
  a.kc = kc.data_ptr(); a.vc = vc.data_ptr();
  a.bias = bias.data_ptr<float>();
  a.n_bias = (int)bias.size(1);
  a.softcap = (float)softcap;
  a.v_norm = true;
  a.table = ints(table, 1, "page table");
  a.max_pages = (int)table.size(1);
  a.size = (int)size; a.keep = size > 0 ? (int)keep : 0;
  a.scale = (float)scale; a.eps = (float)eps; a.out_scale = (float)out_scale;
  attend(a, x, pos, slot, tiles, n_dec, max_len);
}

// rows [q | k | gate, the last if `gated`]; kc (pages, kv, 64, dim) takes k,
// which is the value as well, ks (pages, 64) what its norm divides by
Tensor tied_attention(Tensor x, Tensor kc, Tensor ks, Tensor table, Tensor pos,
                      Tensor slot, Tensor tiles, long n_dec, Tensor qw,
                      Tensor kw, OptTensor slopes, c10::optional<double> sink,
                      double t_coef, long t_every, bool gated, long heads,
                      long size, double scale, double eps, long max_len) {
  const auto ty = x.scalar_type();
  is_f32(x);
  dense(x, "rows"); dense(kc, "cache"); dense(table, "page table");
  TORCH_CHECK(kc.dim() == 4 && table.dim() == 2 && x.dim() == 2, "cache ranks");
  AttnArgs a{};
  a.H = (int)heads;
  a.G = (int)kc.size(1);
  a.dim = a.vdim = (int)kc.size(3);
  TORCH_CHECK(a.G >= 1 && a.H >= 1 && a.H % a.G == 0, "kv heads must divide heads");
  TORCH_CHECK(a.dim >= 1 && a.dim <= 256, "head sizes 1..256 are supported");
  TORCH_CHECK(kc.size(2) == LM_PAGE && kc.scalar_type() == ty, "cache");
  shaped(ks, {kc.size(0), LM_PAGE}, torch::kFloat32, "key factors");
  a.ld = x.size(1);
  const long n = (long)(a.H + a.G) * a.dim + (gated ? (long)a.H * a.dim : 0);
  TORCH_CHECK(a.ld >= n && a.ld % 8 == 0, "row length ", a.ld);
  TORCH_CHECK(size >= 0 && t_every >= 0, "chunk size, temperature");
  const size_t es = x.element_size();
  a.qkv = x.data_ptr(); a.kc = a.vc = kc.data_ptr();
  a.ks = ks.data_ptr<float>();
  if (gated) a.gate = (const char*)a.qkv + (long)(a.H + a.G) * a.dim * es;
  shaped(qw, {(long)a.H * a.dim}, ty, "q norm");
  shaped(kw, {(long)a.G * a.dim}, ty, "k norm");
  a.qw = qw.data_ptr(); a.kw = kw.data_ptr();
  a.slopes = (const float*)opt_vec(slopes, a.H, torch::kFloat32, "slopes");
  a.has_sink = sink.has_value();
  a.out_scale = 1.f;
  a.sink0 = (float)sink.value_or(0.0);
  a.t_coef = (float)t_coef; a.t_every = (int)t_every;
  a.table = ints(table, 1, "page table");
  a.max_pages = (int)table.size(1);
  a.size = (int)size; a.scale = (float)scale; a.eps = (float)eps;
  return attend(a, x, pos, slot, tiles, n_dec, max_len);
}

Tensor retention(Tensor qkvg, Tensor state, Tensor pos, Tensor slot,
                 Tensor tiles, Tensor seqs, long n_dec, Tensor pows, Tensor dec,
                 OptTensor cos_t, OptTensor sin_t, double kscale, double eps,
                 bool light) {
  const bool f32 = is_f32(qkvg);
  dense(qkvg, "qkvg"); dense(state, "state");
  TORCH_CHECK(state.dim() == 4 && state.scalar_type() == torch::kFloat32, "state");
  RetArgs a{};
  a.H = (int)state.size(1);
  a.dv = (int)state.size(2);
  a.dk = (int)state.size(3);
  TORCH_CHECK(a.dk >= 1 && a.dk <= 256 && a.dv >= 1 && a.dv <= 256,
              "head sizes 1..256 are supported");
  TORCH_CHECK(a.H >= 1 && a.H <= 65535, "heads");
  a.ld = 2L * a.H * (a.dk + a.dv);
  TORCH_CHECK(qkvg.dim() == 2 && qkvg.size(1) == a.ld, "qkvg row length");
  shaped(pows, {a.H, LM_TILE + 1}, torch::kFloat32, "decay powers");
  shaped(dec, {a.H, 2}, torch::kFloat32, "decays");
  if (cos_t.has_value()) {
    TORCH_CHECK(sin_t.has_value(), "sin table");
    a.rd = 2 * (int)cos_t->size(1);
    TORCH_CHECK(a.rd <= a.dk, "rotated span exceeds the head");
    shaped(*cos_t, {cos_t->size(0), a.rd / 2}, torch::kFloat32, "cos");
    shaped(*sin_t, {cos_t->size(0), a.rd / 2}, torch::kFloat32, "sin");
    a.cos_t = cos_t->data_ptr<float>();
    a.sin_t = sin_t->data_ptr<float>();
  }
  const long T = qkvg.size(0);
  TORCH_CHECK(n_dec >= 0 && n_dec <= T && n_dec <= 65535, "decode rows");
  const int* pp = ints(pos, T, "positions");
  const int* sp = ints(slot, T, "slots");
  const long nt = tiles.numel() / 4, ns = seqs.numel() / 4;
  const int4* tp = (const int4*)ints(tiles, 4 * nt, "tiles");
  const int4* qp = (const int4*)ints(seqs, 4 * ns, "sequences");
  auto out = torch::empty({T, (long)a.H * a.dv}, qkvg.options());
  a.qkvg = qkvg.data_ptr(); a.state = state.data_ptr<float>();
  a.out = out.data_ptr(); a.pows = pows.data_ptr<float>();
  a.dec = dec.data_ptr<float>();
  a.kscale = (float)kscale; a.eps = (float)eps;
  a.silu = a.raw = light;
  auto st = cur_stream();
  if (n_dec > 0) lm_ret_decode(a, pp, sp, (int)n_dec, f32, st);
  if (nt > 0) {
    TORCH_CHECK(ns >= 1 && ns <= 65535 && nt <= 65535, "prompt portions");
    auto cs = torch::empty({nt, a.H, a.dv, a.dk}, state.options());
    lm_ret_prefill(a, tp, (int)nt, qp, (int)ns, cs.data_ptr<float>(), f32, st);
  }
  launched();
  return out;
}

// Where a ragged batch's rows lie, checked.
struct Plan {
  const int *pos, *slot;
  const int4 *tiles, *seqs;
  int n_dec, n_tiles, n_seqs;
};

Plan plan_of(const Tensor& pos, const Tensor& slot, const Tensor& tiles,
             const Tensor& seqs, long n_dec, long T) {
  TORCH_CHECK(n_dec >= 0 && n_dec <= T && n_dec <= 65535, "decode rows");
  Plan p{};
  const long nt = tiles.numel() / 4, ns = seqs.numel() / 4;
  p.pos = ints(pos, T, "positions");
  p.slot = ints(slot, T, "slots");
  p.tiles = (const int4*)ints(tiles, 4 * nt, "tiles");
  p.seqs = (const int4*)ints(seqs, 4 * ns, "sequences");
  TORCH_CHECK(nt <= 65535 && ns <= 65535 && (nt == 0) == (ns == 0) &&
              (nt > 0) == (n_dec < T), "prompt portions");
  p.n_dec = (int)n_dec;
  p.n_tiles = (int)nt;
  p.n_seqs = (int)ns;
  return p;
}

const void* at(const Tensor& t, long i) {
  return (const char*)t.data_ptr() + i * t.element_size();
}

RaggedRows ragged(const Plan& g, long T) {
  return RaggedRows{g.pos, g.slot, g.tiles, g.seqs, g.n_seqs, g.n_dec, (int)T};
}

// tokens (T,) -> float stream x (T, W); last (slots,) the tokens before
Tensor stream_embed(Tensor tokens, Tensor embed, Tensor pos, Tensor slot,
                    Tensor tiles, Tensor seqs, long n_dec, OptTensor rates,
                    OptTensor pairs, long mul_prev, long mul_cur,
                    OptTensor last) {
  dense(embed, "embed");
  const bool f32 = is_f32(embed);
  const long T = tokens.numel(), W = embed.size(1);
  width_ok(W);
  EmbedArgs a{};
  a.tokens = token_ids(tokens, T);
  a.embed = embed.data_ptr(); a.vocab = embed.size(0); a.W = (int)W;
  if (rates.has_value()) {
    shaped(*rates, {(W + 1) / 2}, torch::kFloat64, "turn rates");
    a.rates = rates->data_ptr<double>();
  }
  if (pairs.has_value()) {
    TORCH_CHECK(pairs->dim() == 2 && pairs->size(0) >= 2 && last.has_value(), "pairs");
    a.buckets = pairs->size(0) - 1;
    shaped(*pairs, {a.buckets + 1, W}, embed.scalar_type(), "pairs");
    dense(*last, "last tokens");
    TORCH_CHECK(last->dim() == 1 && last->scalar_type() == torch::kInt64, "last tokens");
    a.pairs = pairs->data_ptr();
    a.mul_prev = mul_prev; a.mul_cur = mul_cur;
    a.last = (long*)last->data_ptr<int64_t>();
  }
  const Plan g = plan_of(pos, slot, tiles, seqs, n_dec, T);
  auto x = torch::empty({T, W}, embed.options().dtype(torch::kFloat32));
  a.x = x.data_ptr<float>();
  lm_stream_embed(a, ragged(g, T), f32, cur_stream());
  launched();
  return x;
}

// {x + mult * y + add + step, its norm blended with the row before}
std::vector<Tensor> shift_norm(Tensor x, OptTensor y, OptTensor weights,
                               double mult, Tensor nw, OptTensor nb,
                               OptTensor na, bool n_rms, double eps, Tensor pos,
                               Tensor slot, Tensor tiles, Tensor seqs,
                               long n_dec, OptTensor shift, OptTensor state,
                               OptTensor add, OptTensor step) {
  const bool f32 = is_f32(nw);
  const auto ty = nw.scalar_type();
  ShiftArgs a{};
  a.x = stream_x(x);
  const long T = x.size(0), W = x.size(1);
  TORCH_CHECK(!na.has_value(), "a dynamic tanh is not served here");
  a.y = sum_of(y, weights, T, W, ty);
  a.mult = (float)mult;
  a.nxt = norm_of(nw, nb, na, n_rms, W, ty, "norm");
  a.W = (int)W; a.eps = (float)eps;
  if (shift.has_value()) {
    TORCH_CHECK(state.has_value() && state->dim() == 2, "state of the shift");
    a.shift = opt_vec(shift, W, ty, "shift");
    shaped(*state, {state->size(0), W}, torch::kFloat32, "state of the shift");
    a.state = state->data_ptr<float>();
  }
  if (add.has_value()) {
    shaped(*add, {T, W}, torch::kFloat32, "added stream");
    a.add = add->data_ptr<float>();
  }
  a.step = opt_vec(step, W, ty, "step");
  const Plan g = plan_of(pos, slot, tiles, seqs, n_dec, T);
  auto xo = torch::empty_like(x);
  auto h = torch::empty({T, W}, nw.options());
  a.xo = xo.data_ptr<float>(); a.h = h.data_ptr();
  lm_shift_norm(a, ragged(g, T), f32, cur_stream());
  launched();
  return {xo, h};
}

// columns [col, ...) of x: [q | k | v | gate | what makes the decays]; result
// into columns [out_col, ...) of out
void gla(Tensor x, long col, Tensor out, long out_col, Tensor state, Tensor pos,
         Tensor slot, Tensor tiles, Tensor seqs, long n_dec, Tensor a2,
         Tensor a2b, double tau, Tensor norm, double out_scale, double eps) {
  const bool f32 = is_f32(x);
  const auto ty = x.scalar_type();
  dense(x, "rows"); dense(out, "out"); dense(state, "state"); dense(a2, "a2");
  TORCH_CHECK(x.dim() == 2 && out.dim() == 2 && a2.dim() == 2, "ranks");
  TORCH_CHECK(state.dim() == 4 && state.scalar_type() == torch::kFloat32, "state");
  GlaArgs a{};
  a.H = (int)state.size(1);
  a.dv = (int)state.size(2);
  a.dk = (int)state.size(3);
  a.rank = (int)a2.size(1);
  TORCH_CHECK(a.dk >= 1 && a.dk <= 256 && a.dv >= 1 && a.dv <= 256,
              "head sizes 1..256 are supported");
  TORCH_CHECK(a.H >= 1 && a.H <= 65535 && a.rank >= 1, "heads, rank");
  TORCH_CHECK(tau > 0, "tau");
  const long qk = (long)a.H * a.dk, vv = (long)a.H * a.dv, T = x.size(0);
  a.ld = x.size(1); a.ldo = out.size(1);
  TORCH_CHECK(col >= 0 && col % 8 == 0 && a.ld % 8 == 0 &&
              col + 2 * (qk + vv) + a.rank <= a.ld, "row length ", a.ld);
  TORCH_CHECK(out.size(0) == T && out.scalar_type() == ty && out_col >= 0 &&
              out_col + vv <= a.ldo, "out");
  shaped(a2, {qk, a.rank}, ty, "decay matrix");
  shaped(a2b, {qk}, ty, "decay bias");
  shaped(norm, {a.dv}, ty, "norm weight");
  const Plan g = plan_of(pos, slot, tiles, seqs, n_dec, T);
  a.q = at(x, col); a.k = at(x, col + qk); a.v = at(x, col + 2 * qk);
  a.gate = at(x, col + 2 * qk + vv); a.u = at(x, col + 2 * (qk + vv));
  a.a2 = a2.data_ptr(); a.a2b = a2b.data_ptr(); a.norm = norm.data_ptr();
  a.state = state.data_ptr<float>();
  a.out = (char*)out.data_ptr() + out_col * out.element_size();
  a.qscale = 1.0f / std::sqrt((float)a.dk); a.inv_tau = (float)(1.0 / tau);
  a.out_scale = (float)out_scale; a.eps = (float)eps;
  auto st = cur_stream();
  lm_gla_decode(a, g.pos, g.slot, g.n_dec, f32, st);
  if (g.n_tiles > 0) {
    auto ws = torch::empty({lm_gla_scratch(a, g.n_tiles)}, state.options());
    lm_gla_prefill(a, g.tiles, g.n_tiles, g.seqs, g.n_seqs,
                   ws.data_ptr<float>(), f32, st);
  }
  launched();
}

// convolution and silu over columns [col, col + channels) of p
Tensor causal_conv(Tensor p, long col, Tensor w, Tensor b, Tensor tail,
                   Tensor pos, Tensor slot, Tensor tiles, Tensor seqs,
                   long n_dec) {
  dense(p, "p"); dense(w, "kernel"); dense(tail, "tail");
  const bool f32 = is_f32(p);
  const auto ty = p.scalar_type();
  TORCH_CHECK(w.dim() == 2 && w.scalar_type() == ty, "kernel");
  ConvArgs a{};
  a.channels = (int)w.size(0);
  a.taps = (int)w.size(1);
  TORCH_CHECK(a.taps >= 1 && a.taps <= 16, "1 to 16 taps are supported");
  TORCH_CHECK(p.dim() == 2 && col >= 0 && col + a.channels <= p.size(1), "columns");
  shaped(b, {a.channels}, ty, "bias");
  shaped(tail, {tail.size(0), a.taps - 1, a.channels}, torch::kFloat32, "tail");
  const long T = p.size(0);
  const Plan g = plan_of(pos, slot, tiles, seqs, n_dec, T);
  auto out = torch::empty({T, a.channels}, p.options());
  a.in = at(p, col); a.ld = p.size(1);
  a.w = w.data_ptr(); a.b = b.data_ptr();
  a.tail = tail.data_ptr<float>(); a.out = out.data_ptr();
  lm_causal_conv(a, g.pos, g.slot, g.n_dec, g.tiles, g.n_tiles, g.seqs,
                 g.n_seqs, f32, cur_stream());
  launched();
  return out;
}

void gated_sizes(GatedArgs& a, const Tensor& state) {
  dense(state, "state");
  TORCH_CHECK(state.dim() == 4 && state.scalar_type() == torch::kFloat32, "state");
  a.H = (int)state.size(1);
  a.dv = (int)state.size(2);
  a.dk = (int)state.size(3);
  TORCH_CHECK(a.dk >= 1 && a.dk <= 256 && a.dv >= 1 && a.dv <= 256,
              "head and state sizes 1..256 are supported");
  TORCH_CHECK(a.H >= 1 && a.H <= 65535, "heads");
  a.state = state.data_ptr<float>();
}

// p rows [z | x, B, C | step sizes]; xbc the convolved middle part
Tensor mamba2(Tensor p, Tensor xbc, Tensor state, Tensor pos, Tensor slot,
              Tensor tiles, Tensor seqs, long n_dec, long groups,
              Tensor dt_bias, Tensor a_log, Tensor skip) {
  const bool f32 = is_f32(p);
  const auto ty = p.scalar_type();
  dense(p, "p");
  GatedArgs a{};
  gated_sizes(a, state);
  TORCH_CHECK(groups >= 1 && a.H % groups == 0, "groups must divide heads");
  const long T = p.size(0), inner = (long)a.H * a.dv, gn = groups * a.dk;
  const long ch = inner + 2 * gn;
  TORCH_CHECK(p.dim() == 2 && p.size(1) >= inner + ch + a.H, "p row length");
  shaped(xbc, {T, ch}, ty, "xbc");
  shaped(dt_bias, {a.H}, ty, "dt_bias");
  shaped(a_log, {a.H}, ty, "A_log");
  shaped(skip, {a.H}, ty, "D");
  const Plan g = plan_of(pos, slot, tiles, seqs, n_dec, T);
  auto out = torch::empty({T, inner}, p.options());
  a.v = xbc.data_ptr(); a.k = at(xbc, inner); a.q = at(xbc, inner + gn);
  a.ld = ch; a.hpg = (int)(a.H / groups);
  a.gate = p.data_ptr(); a.g0 = at(p, inner + ch); a.ldg = p.size(1);
  a.b0 = dt_bias.data_ptr(); a.b1 = a_log.data_ptr(); a.skip = skip.data_ptr();
  a.qscale = 1.f; a.out = out.data_ptr();
  auto st = cur_stream();
  lm_mamba2_decode(a, g.pos, g.slot, g.n_dec, f32, st);
  if (g.n_tiles > 0) {
    auto ws = torch::empty({lm_gated_scratch(a, g.n_tiles, false)}, state.options());
    lm_mamba2_prefill(a, g.tiles, g.n_tiles, g.seqs, g.n_seqs,
                      ws.data_ptr<float>(), f32, st);
  }
  launched();
  return out;
}

// p rows [q | k | v | output gate | input gate | forget gate]
Tensor mlstm(Tensor p, Tensor state, Tensor n, Tensor m, Tensor pos,
             Tensor slot, Tensor tiles, Tensor seqs, long n_dec, Tensor i_b,
             Tensor f_b, double cap, Tensor norm, double eps) {
  const bool f32 = is_f32(p);
  const auto ty = p.scalar_type();
  dense(p, "p");
  GatedArgs a{};
  gated_sizes(a, state);
  const long T = p.size(0), qk = (long)a.H * a.dk, vv = (long)a.H * a.dv;
  TORCH_CHECK(p.dim() == 2 && p.size(1) >= 2 * (qk + vv + a.H), "p row length");
  shaped(n, {state.size(0), a.H, a.dk}, torch::kFloat32, "normalizer");
  shaped(m, {state.size(0), a.H}, torch::kFloat32, "running maximum");
  shaped(i_b, {a.H}, ty, "input gate bias");
  shaped(f_b, {a.H}, ty, "forget gate bias");
  shaped(norm, {vv}, ty, "norm weight");
  TORCH_CHECK(cap > 0, "gate cap");
  const Plan g = plan_of(pos, slot, tiles, seqs, n_dec, T);
  auto out = torch::empty({T, vv}, p.options());
  a.q = p.data_ptr(); a.k = at(p, qk); a.v = at(p, 2 * qk); a.ld = p.size(1);
  a.hpg = 1;
  a.gate = at(p, 2 * qk + vv); a.g0 = at(p, 2 * (qk + vv));
  a.g1 = at(p, 2 * (qk + vv) + a.H); a.ldg = p.size(1);
  a.b0 = i_b.data_ptr(); a.b1 = f_b.data_ptr(); a.norm = norm.data_ptr();
  a.cap = (float)cap; a.qscale = 1.0f / std::sqrt((float)a.dk);
  a.eps = (float)eps;
  a.n = n.data_ptr<float>(); a.m = m.data_ptr<float>(); a.out = out.data_ptr();
  auto st = cur_stream();
  lm_mlstm_decode(a, g.pos, g.slot, g.n_dec, f32, st);
  if (g.n_tiles > 0) {
    auto ws = torch::empty({lm_gated_scratch(a, g.n_tiles, true)}, state.options());
    lm_mlstm_prefill(a, g.tiles, g.n_tiles, g.seqs, g.n_seqs,
                     ws.data_ptr<float>(), f32, st);
  }
  launched();
  return out;
}

LatentArgs latent_args(const Tensor& a, const Tensor& kc, const Tensor& table,
                       long q_rank, long rank, long rot, const OptTensor& cos_t,
                       const OptTensor& sin_t) {
  dense(a, "a"); dense(kc, "latent cache"); dense(table, "page table");
  TORCH_CHECK(a.dim() == 2 && kc.dim() == 3 && table.dim() == 2, "ranks");
  LatentArgs r{};
  r.a = a.data_ptr(); r.lda = a.size(1);
  r.q_rank = (int)q_rank; r.rank = (int)rank; r.rot = (int)rot;
  r.row = (int)kc.size(2);
  TORCH_CHECK(q_rank >= 1 && rank >= 1 && rot >= 0 && rot <= 256 &&
              q_rank + rank + rot <= a.size(1), "latent sizes");
  TORCH_CHECK(kc.size(1) == LM_PAGE && kc.scalar_type() == a.scalar_type() &&
              r.row == (rank + 7) / 8 * 8 + (rot + 7) / 8 * 8, "latent cache");
  if (cos_t.has_value()) {
    TORCH_CHECK(sin_t.has_value(), "sin table");
    r.rd = 2 * (int)cos_t->size(1);
    TORCH_CHECK(r.rd <= rot, "rotated span exceeds the key part");
    shaped(*cos_t, {cos_t->size(0), r.rd / 2}, torch::kFloat32, "cos");
    shaped(*sin_t, {cos_t->size(0), r.rd / 2}, torch::kFloat32, "sin");
    TORCH_CHECK(cos_t->size(0) >= (table.size(1) - 1) * LM_PAGE + 1, "rotary table length");
    r.cos_t = cos_t->data_ptr<float>();
    r.sin_t = sin_t->data_ptr<float>();
  }
  r.kc = kc.data_ptr();
  r.table = ints(table, 1, "page table");
  r.max_pages = (int)table.size(1);
  return r;
}

// Norms and rotation of the latents of all rows, cached; returns the query
// latents (T, q_rank) and, of `keys`, latents (R, rank) and key parts (R, rot)
std::vector<Tensor> latent_prep(Tensor a, Tensor kc, Tensor table, Tensor pos,
                                Tensor slot, Tensor keys, long n_dec,
                                Tensor qw, Tensor kw, long rot, OptTensor cos_t,
                                OptTensor sin_t, double eps) {
  const bool f32 = is_f32(a);
  const long T = a.size(0), q_rank = qw.numel(), rank = kw.numel();
  LatentArgs r = latent_args(a, kc, table, q_rank, rank, rot, cos_t, sin_t);
  r.eps = (float)eps;
  shaped(qw, {q_rank}, a.scalar_type(), "query norm");
  shaped(kw, {rank}, a.scalar_type(), "key norm");
  TORCH_CHECK(n_dec >= 0 && n_dec <= T, "decode rows");
  const long R = keys.numel() / 4;
  const int* kp = ints(keys, 4 * R, "keys");
  auto cq = torch::empty({T, q_rank}, a.options());
  auto c = torch::empty({R, rank}, a.options());
  auto kr = torch::empty({R, rot}, a.options());
  lm_latent_prep(r, ints(pos, T, "positions"), ints(slot, T, "slots"), (int)T,
                 qw.data_ptr(), kw.data_ptr(), cq.data_ptr(), (const int4*)kp,
                 (int)R, c.data_ptr(), kr.data_ptr(), f32, cur_stream());
  launched();
  return {cq, c, kr};
}

// q (T, H*(dim+rot)) from the query latents; k, v: keys and values expanded
// from the gathered latents.  Rows [0, n_dec) are single new tokens.
Tensor latent_attend(Tensor q, OptTensor k, OptTensor v, Tensor kr, Tensor a,
                     Tensor kc, Tensor table, Tensor pos, Tensor slot,
                     Tensor blocks, long n_dec, Tensor wuk, Tensor wuv,
                     OptTensor cos_t, OptTensor sin_t, long heads, long dim,
                     long vdim, long rot, long q_rank, long size, double scale,
                     long max_len) {
  const bool f32 = is_f32(a);
  const auto ty = a.scalar_type();
  const long T = a.size(0), rank = wuk.size(0);
  LatentArgs r = latent_args(a, kc, table, q_rank, rank, rot, cos_t, sin_t);
  r.H = (int)heads; r.dim = (int)dim; r.vdim = (int)vdim;
  r.size = (int)size; r.scale = (float)scale;
  TORCH_CHECK(heads >= 1 && heads <= 65535 && size >= 0 &&
              q_rank + rank + rot + heads <= a.size(1), "heads");
  TORCH_CHECK(dim >= 1 && vdim >= 1 && vdim <= 256 &&
              (dim + 7) / 8 * 8 + (rot + 7) / 8 * 8 <= 256,
              "head sizes up to 256 are supported");
  shaped(q, {T, heads * (dim + rot)}, ty, "queries");
  shaped(wuk, {rank, heads * dim}, ty, "key matrix");
  shaped(wuv, {heads * vdim, rank}, ty, "value matrix");
  TORCH_CHECK(n_dec >= 0 && n_dec <= T && n_dec <= 65535, "decode rows");
  const int* pp = ints(pos, T, "positions");
  const int* sp = ints(slot, T, "slots");
  auto out = torch::empty({T, heads * vdim}, a.options());
  auto st = cur_stream();
  if (n_dec > 0) {
    TORCH_CHECK(lm_latent_decode_fits(r), "latent size not supported");
    // enough blocks to fill the chip, none with fewer than ~128 keys; the
    // merge takes at most 64 splits
    const long nb = n_dec * ((heads + 15) / 16);
    const long keys = size > 0 ? std::min<long>(size, max_len) : max_len;
    long ns = std::min((512 + nb - 1) / nb, (keys + 127) / 128);
    ns = std::max<long>(1, std::min<long>(ns, 64));
    TORCH_CHECK((keys + ns - 1) / ns <= 1000 * LM_PAGE, "too many keys");
    auto qa = torch::empty({n_dec, heads, r.row}, a.options().dtype(torch::kFloat32));
    auto ws = torch::empty({n_dec * heads * ns * (rank + 2)}, qa.options());
    lm_latent_decode(r, q.data_ptr(), wuk.data_ptr(), wuv.data_ptr(), pp, sp,
                     (int)n_dec, (int)ns, qa.data_ptr<float>(),
                     ws.data_ptr<float>(), out.data_ptr(), f32, st);
  }
  if (n_dec < T) {
    const long nb = blocks.numel() / 4;
    const int* bp = ints(blocks, 4 * nb, "blocks");
    TORCH_CHECK(k.has_value() && v.has_value() && nb >= 1, "keys of the prompts");
    const long R = k->size(0);
    shaped(*k, {R, heads * dim}, ty, "keys");
    shaped(*v, {R, heads * vdim}, ty, "values");
    shaped(kr, {R, rot}, ty, "key parts");
    TORCH_CHECK(nb * heads < (1L << 31), "too many blocks");
    lm_latent_prefill(r, q.data_ptr(), k->data_ptr(), v->data_ptr(),
                      kr.data_ptr(), (const int4*)bp, (int)nb, out.data_ptr(),
                      f32, st);
  }
  launched();
  return out;
}

// x (T, W) times r (n, W) -> float (T, n), for few rows
Tensor router_logits(Tensor x, Tensor r) {
  dense(x, "x");
  TORCH_CHECK(x.dim() == 2 && r.dim() == 2 && x.scalar_type() == torch::kBFloat16 &&
              x.size(1) % 8 == 0 && x.size(0) <= 65535, "bf16 rows of 8k columns");
  shaped(r, {r.size(0), x.size(1)}, torch::kBFloat16, "router");
  auto z = torch::empty({x.size(0), r.size(0)}, x.options().dtype(torch::kFloat32));
  if (z.numel() > 0)
    lm_moe_logits(x.data_ptr(), r.data_ptr(), z.data_ptr<float>(),
                  (int)x.size(0), (int)x.size(1), (int)r.size(0), cur_stream());
  launched();
  return z;
}

// sizes and operands of a routed feed-forward without what chooses
MoeArgs moe_args(const Tensor& x, const Tensor& gu, const Tensor& down,
                 const OptTensor& sgu, const OptTensor& sdown, long top) {
  const auto ty = x.scalar_type();
  dense(x, "x"); dense(gu, "gate and up"); dense(down, "down");
  TORCH_CHECK(x.dim() == 2 && gu.dim() == 3, "ranks");
  MoeArgs a{};
  TORCH_CHECK(x.size(0) < (1L << 30), "too many tokens");
  a.T = (int)x.size(0); a.W = (int)x.size(1);
  a.E = (int)gu.size(0);
  a.ff = (int)gu.size(1) / 2;
  shaped(gu, {a.E, 2L * a.ff, a.W}, ty, "gate and up");
  shaped(down, {a.E, a.W, a.ff}, ty, "down");
  a.top = a.K = (int)top;
  if (sgu.has_value()) {
    TORCH_CHECK(sdown.has_value() && sgu->dim() == 2, "shared expert");
    a.ffs = (int)sgu->size(0) / 2;
    shaped(*sgu, {2L * a.ffs, a.W}, ty, "shared gate and up");
    shaped(*sdown, {a.W, a.ffs}, ty, "shared down");
    a.sgu = sgu->data_ptr(); a.sdown = sdown->data_ptr();
    a.K = a.top + 1;
  }
  TORCH_CHECK(a.E >= 1 && a.E <= LM_MOE_EXPERTS && a.ff >= 1, "experts");
  TORCH_CHECK(top >= 1 && top <= LM_MOE_TOP, "experts per token");
  TORCH_CHECK((long)a.T * a.K < (1L << 30), "too many tokens");
  a.x = x.data_ptr(); a.gu = gu.data_ptr(); a.down = down.data_ptr();
  return a;
}

// chooses and runs; returns the places' outputs y (T, K, W) and their weights
// (T, K)
std::vector<Tensor> moe_run(MoeArgs& a, const Tensor& x) {
  const bool f32 = is_f32(x);
  const long T = a.T;
  a.lda = (std::max(a.ff, a.ffs) + 7) / 8 * 8;
  a.rows = lm_moe_rows(a, f32);
  // each expert's last tile may be short
  const long nt = (T * a.top + a.rows - 1) / a.rows + std::min<long>(a.E, T * a.top) +
                  (a.K > a.top ? (T + a.rows - 1) / a.rows : 0);
  TORCH_CHECK(nt <= 65535, "too many tiles");
  a.n_tiles = (int)nt;
  auto wts = torch::empty({T, a.K}, x.options().dtype(torch::kFloat32));
  auto plan = torch::empty({4 * nt + T * a.K + T * a.top},
                           x.options().dtype(torch::kInt32));
  auto act = torch::empty({T * a.K, (long)a.lda}, x.options());
  auto y = torch::empty({T, (long)a.K, (long)a.W}, x.options());
  a.wts = wts.data_ptr<float>();
  a.tiles = (int4*)plan.data_ptr<int>();
  a.order = plan.data_ptr<int>() + 4 * nt;
  a.ids = a.order + T * a.K;
  a.act = act.data_ptr(); a.y = y.data_ptr();
  lm_moe_plan(a, cur_stream());
  lm_moe_experts(a, f32, cur_stream());
  launched();
  return {y, wts};
}

// z (T, >= E + 1 with a shared expert) router logits, x (T, W)
std::vector<Tensor> moe(Tensor x, Tensor z, Tensor gu, Tensor down,
                        OptTensor sgu, OptTensor sdown, long top, long groups,
                        long keep, double scale) {
  MoeArgs a = moe_args(x, gu, down, sgu, sdown, top);
  dense(z, "router logits");
  TORCH_CHECK(z.dim() == 2, "ranks");
  TORCH_CHECK(groups >= 1 && groups <= LM_MOE_GROUPS && a.E % groups == 0 &&
              keep >= 1 && keep <= groups, "expert groups");
  TORCH_CHECK(top <= keep * (a.E / groups), "too few experts to choose from");
  a.ldz = (int)z.size(1);
  TORCH_CHECK(z.size(0) == a.T && a.ldz >= a.E + (a.K - a.top) &&
              z.scalar_type() == torch::kFloat32, "router logits");
  a.groups = (int)groups; a.keep = (int)keep; a.scale = (float)scale;
  a.z = z.data_ptr<float>();
  return moe_run(a, x);
}

// table (vocab, top): the experts of each token id
std::vector<Tensor> table_moe(Tensor x, Tensor tokens, Tensor table, Tensor gu,
                              Tensor down) {
  TORCH_CHECK(table.dim() == 2 && table.size(0) >= 1, "table");
  MoeArgs a = moe_args(x, gu, down, c10::nullopt, c10::nullopt, table.size(1));
  a.tokens = token_ids(tokens, a.T);
  a.vocab = table.size(0);
  a.table = ints(table, table.numel(), "table");
  return moe_run(a, x);
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.attr("PAGE") = LM_PAGE;
  m.attr("TILE") = LM_TILE;
  m.def("embed_norm", &embed_norm, "embedding lookup + first norm");
  m.def("residual_norm", &residual_norm,
        "post-norm, residual add and next pre-norm in one pass");
  m.def("gelu_erf", &gelu_erf, "exact GELU");
  m.def("paged_attention", &paged_attention,
        "chunked causal attention with sink over a paged cache");
  m.def("window_attention", &window_attention,
        "window attention with kept first tokens over a paged cache");
  m.def("gla", &gla, "gated linear attention over state slots");
  m.def("gated_rms", &gated_rms, "RMS norm of rows behind a sigmoid gate");
  m.def("stream_embed", &stream_embed, "embeddings, positions and pairs");
  m.def("shift_norm", &shift_norm,
        "residual add and a norm blended with the token before");
  m.def("table_moe", &table_moe, "experts by token id");
  m.def("retention", &retention, "retention over state slots");
  m.def("residual_concat", &residual_concat,
        "residual add, then the stream beside the embeddings");
  m.def("replace_norm", &replace_norm, "a new stream and its norm");
  m.def("geglu_tanh", &geglu_tanh, "gelu(gate) * up, tanh form");
  m.def("clamped_glu", &clamped_glu, "clamped gated activation");
  m.def("tied_attention", &tied_attention,
        "attention whose values are its keys over a paged cache");
  m.def("router_logits", &router_logits, "router logits of few tokens");
  m.def("moe", &moe, "routed experts and a shared one");
  m.def("softcap", &softcap, "cap * tanh(x / cap)");
  m.def("grouped_rms", &grouped_rms, "RMS norm of equal parts of a row");
  m.def("causal_conv", &causal_conv, "short convolution over state slots");
  m.def("mamba2", &mamba2, "state-space recurrence over state slots");
  m.def("mlstm", &mlstm, "matrix memory over state slots");
  m.def("latent_prep", &latent_prep, "latents of a batch, cached and gathered");
  m.def("latent_attend", &latent_attend,
        "sliding-window attention over cached latents");
}
