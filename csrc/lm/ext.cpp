// pybind11 layer of the mixer-stack serving kernels: every shape, dtype and
// range that a kernel relies on is checked here, on the host.
#include <torch/extension.h>
#include <c10/hip/HIPStream.h>

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

// tokens (T,) -> x (T, W) float stream, returns its norm h (T, W)
std::vector<Tensor> embed_norm(Tensor tokens, Tensor embed, Tensor w,
                               OptTensor b, double eps) {
  dense(tokens, "tokens"); dense(embed, "embed");
  const bool f32 = is_f32(embed);
  const auto ty = embed.scalar_type();
  const long T = tokens.numel(), V = embed.size(0), W = embed.size(1);
  TORCH_CHECK(tokens.scalar_type() == torch::kInt64, "tokens must be int64");
  width_ok(W);
  shaped(w, {W}, ty, "norm weight");
  auto x = torch::empty({T, W}, embed.options().dtype(torch::kFloat32));
  auto h = torch::empty({T, W}, embed.options());
  lm_embed_norm(tokens.data_ptr<int64_t>(), embed.data_ptr(), x.data_ptr<float>(),
                w.data_ptr(), opt_vec(b, W, ty, "norm bias"), h.data_ptr(),
                (int)T, (int)W, V, (float)eps, f32, cur_stream());
  launched();
  return {x, h};
}

// x += mult * LN(y; pw, pb); returns LN(x; nw, nb) of `rows` (or all rows)
Tensor residual_norm(Tensor x, OptTensor y, OptTensor pw, OptTensor pb,
                     double mult, Tensor nw, OptTensor nb, OptTensor rows,
                     double eps, bool store_x) {
  dense(x, "x"); dense(nw, "norm weight");
  const bool f32 = is_f32(nw);
  const auto ty = nw.scalar_type();
  const long T = x.size(0), W = x.size(1);
  width_ok(W);
  TORCH_CHECK(x.scalar_type() == torch::kFloat32, "the stream is float32");
  shaped(nw, {W}, ty, "norm weight");
  if (y.has_value()) shaped(*y, {T, W}, ty, "sublayer output");
  long n = T;
  const int* rp = nullptr;
  if (rows.has_value()) {
    n = rows->numel();
    rp = ints(*rows, n, "rows");
    TORCH_CHECK(!store_x, "a row subset leaves the stream alone");
  }
  auto h = torch::empty({n, W}, nw.options());
  lm_residual_norm(x.data_ptr<float>(), y.has_value() ? y->data_ptr() : nullptr,
                   opt_vec(pw, W, ty, "post norm weight"),
                   opt_vec(pb, W, ty, "post norm bias"), (float)mult,
                   nw.data_ptr(), opt_vec(nb, W, ty, "norm bias"), h.data_ptr(),
                   rp, (int)n, (int)W, (float)eps, store_x, f32, cur_stream());
  launched();
  return h;
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
                   const OptTensor& sink, long heads, long size, double scale,
                   double eps) {
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
  a.table = ints(table, 1, "page table");
  a.max_pages = (int)table.size(1);
  a.size = (int)size; a.scale = (float)scale; a.eps = (float)eps;
  return a;
}

// Rows [0, n_dec) of qkv are single new tokens, the rest prompt portions
// described by `tiles`; returns (T, heads * vdim).
Tensor paged_attention(Tensor qkv, Tensor kc, Tensor vc, Tensor table,
                       Tensor pos, Tensor slot, Tensor tiles, long n_dec,
                       OptTensor qw, OptTensor kw, OptTensor sink, long heads,
                       long size, double scale, double eps, long max_len) {
  const bool f32 = is_f32(qkv);
  AttnArgs a = attn_args(qkv, kc, vc, table, qw, kw, sink, heads, size, scale, eps);
  const long T = qkv.size(0);
  TORCH_CHECK(n_dec >= 0 && n_dec <= T, "decode rows");
  const int* pp = ints(pos, T, "positions");
  const int* sp = ints(slot, T, "slots");
  const long nt = tiles.numel() / 4;
  const int4* tp = (const int4*)ints(tiles, 4 * nt, "tiles");
  auto out = torch::empty({T, (long)a.H * a.vdim}, qkv.options());
  a.out = out.data_ptr();
  auto st = cur_stream();
  if (n_dec > 0) {
    TORCH_CHECK(n_dec <= 65535, "too many decode rows");
    // enough blocks to fill the chip, none with fewer than ~128 keys;
    // the merge takes at most 64 splits
    const long hg = a.H / a.G, hc = hg <= 2 ? hg : 4;
    const long blocks = n_dec * a.G * ((hg + hc - 1) / hc);
    const long keys = size > 0 ? std::min<long>(size, max_len) : max_len;
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

Tensor retention(Tensor qkvg, Tensor state, Tensor pos, Tensor slot,
                 Tensor tiles, Tensor seqs, long n_dec, Tensor pows, Tensor dec,
                 OptTensor cos_t, OptTensor sin_t, double kscale, double eps) {
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
  m.def("retention", &retention, "retention over state slots");
}
