// Residual-stream kernels: the stream x stays float in HBM and is touched
// once per sublayer.  One launch applies the norm after a sublayer, adds
// it to the stream and produces the next sublayer's normed input:
//     x <- x + mult * N(y; post)         h <- N(x; next)
// so a layer costs two reads and one write of x instead of four passes.
// N is a layer norm, an RMS norm, tanh(alpha * x) * w + b where an alpha is
// given, or nothing (h <- x).  y may be given as `mix` rows per row and
// their float weights: the experts' outputs of a routed feed-forward.
// Two more forms serve a span whose input is a projection: h <- [x; e]
// with the tokens' embeddings e, and x <- y + step.
//
// Rows up to 2048 wide take one wave each (4 rows a block, shuffles
// only); wider rows, and few rows that are not narrow, take a 4-wave block.

#include "norm.h"

namespace {

// tanh(alpha * v), what a dynamic tanh has in place of statistics
template <int VEC, int NV>
DEVINL void tanh_rows(Pack<VEC> (&v)[NV], float alpha) {
  #pragma unroll
  for (int i = 0; i < NV; ++i)
    #pragma unroll
    for (int j = 0; j < VEC; ++j) v[i].v[j] = tanhf(alpha * v[i].v[j]);
}

struct NormArgs {
  const long* tokens;   // embedding form: x <- embed[token]
  const void* embed;
  long vocab;
  const void* ptab;     // embedding form: learned positions or null
  const int* pos;
  int n_pos;
  float* x;
  const void* y;        // sublayer output or null
  const float* mw;      // null: y is [T][W]; else y is [T][mix][W] and these
  int mix;              // are the weights [T][mix] of its rows
  const void* pw;       // its norm (null: y is added as it is)
  const void* pb;
  const void* pa;       // its alpha: dynamic tanh (null: layer or RMS norm)
  bool p_rms, p_one, n_one;   // *_one: a single weight for all columns
  float mult;
  const void* nw;       // next norm or null
  const void* nb;
  const void* na;
  bool n_rms;
  void* h;              // null: not wanted
  const void* step;     // replacing form: x <- y + step
  bool y_f32;           // y is float whatever the weights are (replacing form)
  bool cat;             // h <- [x; embed[token]] (rows of 2 W), x as usual
  const int* rows;      // null: identity; else h[r] comes from x[rows[r]]
  int T, W;
  float eps;
  bool store_x;
};

template <bool F32, int TPR, int VEC, int NV>
__global__ void __launch_bounds__(256)
residual_norm_kernel(NormArgs a) {
  __shared__ float red[4];
  constexpr int RPB = 256 / TPR;
  const int tid = threadIdx.x % TPR;
  const int out_row = blockIdx.x * RPB + threadIdx.x / TPR;
  if (out_row >= a.T) return;     // whole wave (TPR 64) or whole block
  const long row = a.rows ? a.rows[out_row] : out_row;
  const int W = a.W;

  // the weights of a narrow share are fetched with the row, so that the
  // reductions wait for one memory round trip and not for three
  constexpr bool EARLY = NV <= 4;
  Held<F32, VEC> wp[EARLY ? NV : 1], bp[EARLY ? NV : 1], wn[EARLY ? NV : 1],
      bn[EARLY ? NV : 1];
  if constexpr (EARLY) {
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      wp[i] = bp[i] = wn[i] = bn[i] = Held<F32, VEC>{};
      if (c < W) {
        if (a.pw) wp[i].load_weight(a.pw, c, a.p_one);
        if (a.pb) bp[i].load(a.pb, c);
        if (a.nw) wn[i].load_weight(a.nw, c, a.n_one);
        if (a.nb) bn[i].load(a.nb, c);
      }
    }
  }

  Pack<VEC> x[NV];
  if (a.step) {
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      x[i] = Pack<VEC>{};
      if (c < W) {
        const Pack<VEC> s = ldv<F32, VEC>(a.step, c);
        x[i] = a.y_f32 ? ldv<true, VEC>(a.y, row * W + c)
                       : ldv<F32, VEC>(a.y, row * W + c);
        #pragma unroll
        for (int j = 0; j < VEC; ++j) x[i].v[j] += s.v[j];
        stv<true, VEC>(a.x, row * W + c, x[i]);
      }
    }
  } else if (a.tokens && !a.cat) {
    const long tok = a.tokens[row];
    const bool ok = tok >= 0 && tok < a.vocab;
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      x[i] = Pack<VEC>{};
      if (c < W && ok) x[i] = ldv<F32, VEC>(a.embed, tok * W + c);
      if (c < W && a.ptab) {
        const int p = a.pos[row];
        if (p >= 0 && p < a.n_pos) {
          const Pack<VEC> e = ldv<F32, VEC>(a.ptab, (long)p * W + c);
          #pragma unroll
          for (int j = 0; j < VEC; ++j) x[i].v[j] += e.v[j];
        }
      }
      if (c < W) stv<true, VEC>(a.x, row * W + c, x[i]);
    }
  } else {
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      x[i] = Pack<VEC>{};
      if (c < W) x[i] = ldv<true, VEC>(a.x, row * W + c);
    }
  }
  if (a.y && !a.step) {
    Pack<VEC> y[NV];
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      y[i] = Pack<VEC>{};
      if (c < W && !a.mw) y[i] = ldv<F32, VEC>(a.y, row * W + c);
    }
    if (a.mw) {
      // CH parts at a time, their loads in flight together
      constexpr int CH = NV <= 4 ? 6 : NV <= 8 ? 3 : 1;
      for (int k0 = 0; k0 < a.mix; k0 += CH) {
        Held<F32, VEC> t[CH][NV];
        float wt[CH];
        #pragma unroll
        for (int k = 0; k < CH; ++k) {
          const bool on = k0 + k < a.mix;
          const long r = row * a.mix + (on ? k0 + k : 0);
          wt[k] = a.mw[r];
          if (!on) wt[k] = 0.f;
          #pragma unroll
          for (int i = 0; i < NV; ++i) {
            const int c = (i * TPR + tid) * VEC;
            t[k][i] = Held<F32, VEC>{};
            if (c < W && on) t[k][i].load(a.y, r * W + c);
          }
        }
        #pragma unroll
        for (int k = 0; k < CH; ++k)
          #pragma unroll
          for (int i = 0; i < NV; ++i) {
            const Pack<VEC> u = t[k][i].up();
            #pragma unroll
            for (int j = 0; j < VEC; ++j)
              y[i].v[j] = fmaf(wt[k], u.v[j], y[i].v[j]);
          }
      }
    }
    if (a.pa)
      tanh_rows<VEC, NV>(y, Num<F32>::up(*(const typename Num<F32>::E*)a.pa));
    else if (a.pw)
      layer_norm_rows<TPR, VEC, NV>(y, tid, W, a.eps, a.p_rms, red);
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      if (c < W) {
        if (a.pw) {
          Pack<VEC> w, b{};
          if constexpr (EARLY) {
            w = wp[i].up();
            b = bp[i].up();
          } else {
            Held<F32, VEC> t;
            t.load_weight(a.pw, c, a.p_one);
            w = t.up();
            if (a.pb) b = ldv<F32, VEC>(a.pb, c);
          }
          #pragma unroll
          for (int j = 0; j < VEC; ++j)
            y[i].v[j] = y[i].v[j] * w.v[j] + b.v[j];
        }
        #pragma unroll
        for (int j = 0; j < VEC; ++j) x[i].v[j] += a.mult * y[i].v[j];
        if (a.store_x) stv<true, VEC>(a.x, row * W + c, x[i]);
      }
    }
  }
  if (a.cat) {
    const long tok = a.tokens[row];
    const bool ok = tok >= 0 && tok < a.vocab;
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      if (c < W) {
        Pack<VEC> e{};
        if (ok) e = ldv<F32, VEC>(a.embed, tok * W + c);
        stv<F32, VEC>(a.h, 2 * row * W + c, x[i]);
        stv<F32, VEC>(a.h, (2 * row + 1) * W + c, e);
      }
    }
  }
  if (a.nw) {
    if (a.na)
      tanh_rows<VEC, NV>(x, Num<F32>::up(*(const typename Num<F32>::E*)a.na));
    else
      layer_norm_rows<TPR, VEC, NV>(x, tid, W, a.eps, a.n_rms, red);
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      if (c < W) {
        Pack<VEC> w, b{};
        if constexpr (EARLY) {
          w = wn[i].up();
          b = bn[i].up();
        } else {
          Held<F32, VEC> t;
          t.load_weight(a.nw, c, a.n_one);
          w = t.up();
          if (a.nb) b = ldv<F32, VEC>(a.nb, c);
        }
        #pragma unroll
        for (int j = 0; j < VEC; ++j)
          x[i].v[j] = x[i].v[j] * w.v[j] + b.v[j];
        stv<F32, VEC>(a.h, (long)out_row * W + c, x[i]);
      }
    }
  } else if (a.h && !a.cat) {
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      if (c < W) stv<F32, VEC>(a.h, (long)out_row * W + c, x[i]);
    }
  }
}

template <bool F32, int VEC>
void launch_norm(const NormArgs& a, hipStream_t st) {
  #define LN_GO(TPR, NV)                                                       \
    hipLaunchKernelGGL((residual_norm_kernel<F32, TPR, VEC, NV>),              \
                       dim3((a.T * TPR + 255) / 256), dim3(256), 0, st, a)
  // a block per row where there are too few rows for a wave per row
  if (a.T <= 512 && a.W > 256 * VEC && a.W <= 512 * VEC) LN_GO(256, 2);
  else if (a.W <= 64 * VEC) LN_GO(64, 1);
  else if (a.W <= 128 * VEC) LN_GO(64, 2);
  else if (a.W <= 256 * VEC) LN_GO(64, 4);
  else if (a.W <= 512 * VEC) LN_GO(64, 8);
  else if (a.W <= 1024 * VEC) LN_GO(256, 4);
  else if (a.W <= 2048 * VEC) LN_GO(256, 8);
  else LN_GO(256, 16);            // up to 4096 * VEC (checked by the caller)
  #undef LN_GO
}

void dispatch_norm(const NormArgs& a, bool f32, hipStream_t st) {
  if (a.T <= 0) return;
  const bool v4 = a.W % 4 == 0;
  if (f32) v4 ? launch_norm<true, 4>(a, st) : launch_norm<true, 1>(a, st);
  else v4 ? launch_norm<false, 4>(a, st) : launch_norm<false, 1>(a, st);
}

template <bool F32>
__global__ void __launch_bounds__(256)
gelu_erf_kernel(const void* in, void* out, long n4, long n) {
  const long step = grid_stride();
  auto f = [](float z) { return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f)); };
  for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < n4; i += step) {
    Pack<4> p = ldv<F32, 4>(in, i * 4);
    #pragma unroll
    for (int j = 0; j < 4; ++j) p.v[j] = f(p.v[j]);
    stv<F32, 4>(out, i * 4, p);
  }
  const long tail = n4 * 4 + (long)blockIdx.x * 256 + threadIdx.x;
  if (tail < n) {
    Pack<1> p = ldv<F32, 1>(in, tail);
    p.v[0] = f(p.v[0]);
    stv<F32, 1>(out, tail, p);
  }
}

// act(g) * u of rows [g | u], each n wide
//   GELU_TANH  gelu(g) u, tanh form: 0.5 (1 + tanh(z)) = 1 / (1 + exp(-2 z))
//   CLAMPED    g' sigmoid(alpha g') (u' + shift), g' = min(g, limit),
//              u' = clamp(u, -limit, limit)
struct GateArgs {
  float limit, alpha, shift;
};
template <int ACT>
DEVINL float gate_act(float g, float u, const GateArgs& a) {
  if constexpr (ACT == LM_GELU_TANH) {
    const float t = 1.5957691216057308f * (g + 0.044715f * g * g * g);
    return u * (g / (1.0f + expf(-t)));
  } else {
    const float z = fminf(g, a.limit);
    const float v = fminf(fmaxf(u, -a.limit), a.limit) + a.shift;
    return v * (z / (1.0f + expf(-a.alpha * z)));
  }
}

template <bool F32, int VEC, int ACT>
__global__ void __launch_bounds__(256)
gated_act_kernel(const void* in, void* out, long units, int n, GateArgs a) {
  const long step = grid_stride();
  const int per = n / VEC;
  for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < units; i += step) {
    const long row = i / per, c = (i % per) * VEC;
    const Pack<VEC> g = ldv<F32, VEC>(in, 2 * row * n + c);
    Pack<VEC> u = ldv<F32, VEC>(in, (2 * row + 1) * n + c);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) u.v[j] = gate_act<ACT>(g.v[j], u.v[j], a);
    stv<F32, VEC>(out, row * n + c, u);
  }
}

// cap * tanh(x / cap), float out
template <bool F32>
__global__ void __launch_bounds__(256)
softcap_kernel(const void* in, float* out, long n4, long n, float cap) {
  const long step = grid_stride();
  const float inv = 1.0f / cap;
  for (long i = (long)blockIdx.x * 256 + threadIdx.x; i < n4; i += step) {
    Pack<4> p = ldv<F32, 4>(in, i * 4);
    #pragma unroll
    for (int j = 0; j < 4; ++j) p.v[j] = cap * tanhf(p.v[j] * inv);
    stv<true, 4>(out, i * 4, p);
  }
  const long tail = n4 * 4 + (long)blockIdx.x * 256 + threadIdx.x;
  if (tail < n) {
    Pack<1> p = ldv<F32, 1>(in, tail);
    out[tail] = cap * tanhf(p.v[0] * inv);
  }
}

// y * inv_rms(y) * w (* sigmoid(gate)) over equal parts of a row, one block
// per (row, part); gate: rows of stride ldg, or null
template <bool F32, int VEC>
__global__ void __launch_bounds__(256)
grouped_rms_kernel(const void* __restrict__ y, const void* __restrict__ w,
                   const void* __restrict__ gate, long ldg,
                   void* __restrict__ out, int parts, int n, float eps) {
  __shared__ float red[4];
  const long off = (long)blockIdx.x * n;
  const long woff = (long)(blockIdx.x % parts) * n;
  const long goff = blockIdx.x / parts * ldg + woff;
  float q = 0.f;
  for (int c = threadIdx.x * VEC; c < n; c += 256 * VEC) {
    const Pack<VEC> v = ldv<F32, VEC>(y, off + c);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) q += v.v[j] * v.v[j];
  }
  const float inv = 1.0f / sqrtf(row_sum<256>(q, red) / (float)n + eps);
  for (int c = threadIdx.x * VEC; c < n; c += 256 * VEC) {
    Pack<VEC> v = ldv<F32, VEC>(y, off + c);
    const Pack<VEC> g = ldv<F32, VEC>(w, woff + c);
    Pack<VEC> z;
    if (gate) z = ldv<F32, VEC>(gate, goff + c);
    #pragma unroll
    for (int j = 0; j < VEC; ++j) {
      v.v[j] *= inv * g.v[j];
      if (gate) v.v[j] /= 1.0f + expf(-z.v[j]);
    }
    stv<F32, VEC>(out, off + c, v);
  }
}

}  // namespace

void lm_embed_norm(const long* tokens, const void* embed, const int* pos,
                   const void* ptab, int n_pos, float* x, LmNorm nxt, void* h,
                   int T, int W, long vocab, float eps, bool f32,
                   hipStream_t stream) {
  NormArgs a{};
  a.tokens = tokens; a.embed = embed; a.vocab = vocab;
  a.pos = pos; a.ptab = ptab; a.n_pos = n_pos;
  a.x = x; a.nw = nxt.w; a.nb = nxt.b; a.na = nxt.alpha; a.n_rms = nxt.rms; a.n_one = nxt.one;
  a.h = h; a.T = T; a.W = W; a.eps = eps;
  dispatch_norm(a, f32, stream);
}

void lm_residual_norm(float* x, LmSum y, LmNorm post, float mult,
                      LmNorm nxt, void* h, const int* rows, int T, int W,
                      float eps, bool store_x, bool f32, hipStream_t stream) {
  NormArgs a{};
  a.x = x; a.y = y.y; a.mw = y.w; a.mix = y.n; a.pw = post.w; a.pb = post.b; a.pa = post.alpha; a.p_rms = post.rms; a.p_one = post.one;
  a.mult = mult; a.nw = nxt.w; a.nb = nxt.b; a.na = nxt.alpha; a.n_rms = nxt.rms; a.n_one = nxt.one;
  a.h = h; a.rows = rows; a.T = T; a.W = W; a.eps = eps; a.store_x = store_x;
  dispatch_norm(a, f32, stream);
}

void lm_residual_concat(float* x, LmSum y, LmNorm post, float mult,
                        const long* tokens, const void* embed, void* h, int T,
                        int W, long vocab, float eps, bool f32,
                        hipStream_t stream) {
  NormArgs a{};
  a.x = x; a.y = y.y; a.mw = y.w; a.mix = y.n; a.pw = post.w; a.pb = post.b; a.pa = post.alpha; a.p_rms = post.rms; a.p_one = post.one;
  a.mult = mult; a.tokens = tokens; a.embed = embed; a.vocab = vocab;
  a.cat = true; a.h = h; a.T = T; a.W = W; a.eps = eps; a.store_x = true;
  dispatch_norm(a, f32, stream);
}

void lm_replace_norm(float* x, const void* y, bool y_f32, const void* step,
                     LmNorm nxt, void* h, int T, int W, float eps, bool f32,
                     hipStream_t stream) {
  NormArgs a{};
  a.x = x; a.y = y; a.y_f32 = y_f32; a.step = step;
  a.nw = nxt.w; a.nb = nxt.b; a.na = nxt.alpha; a.n_rms = nxt.rms; a.n_one = nxt.one;
  a.h = h; a.T = T; a.W = W; a.eps = eps;
  dispatch_norm(a, f32, stream);
}

void lm_gelu_erf(const void* in, void* out, long n, bool f32,
                 hipStream_t stream) {
  if (n <= 0) return;
  const long n4 = n / 4;
  const dim3 grid(capped_blocks(std::max<long>(n4, 256), 256, 4096));
  if (f32)
    hipLaunchKernelGGL((gelu_erf_kernel<true>), grid, dim3(256), 0, stream, in, out, n4, n);
  else
    hipLaunchKernelGGL((gelu_erf_kernel<false>), grid, dim3(256), 0, stream, in, out, n4, n);
}

void lm_gated_act(const void* in, void* out, long rows, int n, int act,
                  float limit, float alpha, float shift, bool f32,
                  hipStream_t stream) {
  if (rows <= 0) return;
  const bool v4 = n % 4 == 0;
  const long units = rows * (v4 ? n / 4 : n);
  const dim3 grid(capped_blocks(units, 256, 4096));
  const GateArgs a{limit, alpha, shift};
  #define GG_GO(F, V)                                                          \
    if (act == LM_GELU_TANH)                                                   \
      hipLaunchKernelGGL((gated_act_kernel<F, V, LM_GELU_TANH>), grid,         \
                         dim3(256), 0, stream, in, out, units, n, a);          \
    else                                                                       \
      hipLaunchKernelGGL((gated_act_kernel<F, V, LM_CLAMPED>), grid,           \
                         dim3(256), 0, stream, in, out, units, n, a)
  if (f32 && v4) { GG_GO(true, 4); }
  else if (f32) { GG_GO(true, 1); }
  else if (v4) { GG_GO(false, 4); }
  else { GG_GO(false, 1); }
  #undef GG_GO
}

void lm_softcap(const void* in, float* out, long n, float cap, bool f32,
                hipStream_t stream) {
  if (n <= 0) return;
  const long n4 = n / 4;
  const dim3 grid(capped_blocks(std::max<long>(n4, 256), 256, 4096));
  if (f32)
    hipLaunchKernelGGL((softcap_kernel<true>), grid, dim3(256), 0, stream, in, out, n4, n, cap);
  else
    hipLaunchKernelGGL((softcap_kernel<false>), grid, dim3(256), 0, stream, in, out, n4, n, cap);
}

void lm_grouped_rms(const void* y, const void* w, const void* gate, long ldg,
                    void* out, long rows, int parts, int n, float eps, bool f32,
                    hipStream_t stream) {
  if (rows <= 0) return;
  const dim3 grid((unsigned)(rows * parts));
  // vectors need every row's start aligned
  const bool v4 = n % 4 == 0 && (!gate || (ldg % 4 == 0 && (size_t)gate % 16 == 0));
  #define GR_GO(F, V)                                                          \
    hipLaunchKernelGGL((grouped_rms_kernel<F, V>), grid, dim3(256), 0, stream, \
                       y, w, gate, ldg, out, parts, n, eps)
  if (f32 && v4) GR_GO(true, 4);
  else if (f32) GR_GO(true, 1);
  else if (v4) GR_GO(false, 4);
  else GR_GO(false, 1);
  #undef GR_GO
}
