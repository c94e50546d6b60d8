// The start of a residual stream and norms that look a token back.
//
//  embed: embedding + a sinusoidal position vector + a row per pair of
//    neighbouring tokens.  Angles are turns in double, reduced before they
//    become float, so a position's vector does not lose digits with distance.
//  shift: x' = x + mult * y + add + step, h = norm(x'), and the output
//    h + (h_before - h) * shift.  In prompts a thread group walks some
//    consecutive rows and carries the last h in registers; its first row's
//    predecessor it computes once more.  The new stream goes to another buffer,
//    so that this never meets a row that its own group has already replaced.
//    A single token's predecessor is what its slot keeps.
//
// What a sequence keeps for its next step (its last token, its last h) is
// read and replaced by whoever has the first row of its portion: that group
// computes the portion's last row as well, and nobody else touches the slot.

#include "norm.h"

namespace {

// last row of the portion that `slot` has in this batch; a whole wave asks
DEVINL int last_row(const RaggedRows& r, int slot) {
  const int l = threadIdx.x & 63;
  for (int k0 = 0; k0 < r.n_seqs; k0 += 64) {
    const int k = min(k0 + l, r.n_seqs - 1);
    const int4 q = r.seqs[k];
    const unsigned long long m = __ballot(k0 + l < r.n_seqs && q.w == slot);
    if (m == 0) continue;
    const int at = __ffsll((unsigned long long)m) - 1;
    const int4 t = r.tiles[__shfl(q.x + q.y - 1, at, 64)];
    return t.x + t.y - 1;
  }
  return -1;
}

// whether a row is the first of what its sequence brings
DEVINL bool starts(const RaggedRows& r, int row) {
  return row <= r.n_dec || r.slot[row - 1] != r.slot[row];
}

template <bool F32, int VEC>
__global__ void __launch_bounds__(256)
stream_embed_kernel(EmbedArgs a, RaggedRows r) {
  const int row = blockIdx.x, W = a.W;
  const long tok = a.tokens[row];
  const int p = r.pos[row], s = r.slot[row];
  const bool ok = tok >= 0 && tok < a.vocab;
  long pair = a.buckets;
  if (a.pairs) {
    const bool first = starts(r, row);
    if (p > 0 && s >= 0) {
      const long prev = first ? a.last[s] : a.tokens[row - 1];
      pair = (prev * a.mul_prev + tok * a.mul_cur) % a.buckets;
      if (pair < 0) pair += a.buckets;
    }
    if (first && s >= 0) {                    // uniform
      const int end = row < r.n_dec ? row : last_row(r, s);
      __syncthreads();                        // every thread has read it
      if (threadIdx.x == 0 && end >= 0) a.last[s] = a.tokens[end];
    }
  }
  for (int c = threadIdx.x * VEC; c < W; c += 256 * VEC) {
    Pack<VEC> x{};
    if (ok) x = ldv<F32, VEC>(a.embed, tok * W + c);
    if (a.pairs) {
      const Pack<VEC> b = ldv<F32, VEC>(a.pairs, pair * W + c);
      #pragma unroll
      for (int j = 0; j < VEC; ++j) x.v[j] += b.v[j];
    }
    if (a.rates) {
      #pragma unroll
      for (int j = 0; j < VEC; j += 2) {
        const double t = (double)p * a.rates[(c + j) / 2];
        float sn, cs;
        sincospif((float)(2.0 * (t - floor(t))), &sn, &cs);
        if constexpr (VEC == 1) {
          x.v[0] += c & 1 ? cs : sn;
        } else {
          x.v[j] += sn;
          x.v[j + 1] += cs;
        }
      }
    }
    stv<true, VEC>(a.x, (long)row * W + c, x);
  }
}

// WALK: groups of `per` rows of the portions; else a single token each
template <bool F32, int TPR, int VEC, int NV, bool WALK>
__global__ void __launch_bounds__(256)
shift_norm_kernel(ShiftArgs a, RaggedRows r, int per) {
  __shared__ float red[4];
  const int tid = threadIdx.x % TPR, W = a.W;
  // with a block per row everything that depends on the row alone is uniform
  const int task = TPR == 256 ? blockIdx.x
                              : blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
  const int row0 = WALK ? r.n_dec + task * per : task;
  const int rows = WALK ? min(per, r.T - row0) : task < r.n_dec;
  if (rows <= 0) return;              // whole wave (TPR 64) or whole block

  Held<F32, VEC> wn[NV], mix[NV];
  #pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = (i * TPR + tid) * VEC;
    wn[i] = mix[i] = Held<F32, VEC>{};
    if (c < W) {
      wn[i].load_weight(a.nxt.w, c, a.nxt.one);
      if (a.shift) mix[i].load(a.shift, c);
    }
  }

  // a row's new stream and its norm; also() is called when the loads are out
  auto make = [&](long row, bool store, Pack<VEC> (&h)[NV], auto also) {
    constexpr int CH = NV <= 4 ? 6 : NV <= 8 ? 2 : 1;  // loads in flight
    Held<F32, VEC> t[CH][NV];
    const int n = a.y.y ? (a.y.w ? a.y.n : 1) : 0;
    float wt[CH];
    auto fetch = [&](int k0) {
      #pragma unroll
      for (int k = 0; k < CH; ++k) {
        const bool on = k0 + k < n;
        const long part = row * n + (on ? k0 + k : 0);
        wt[k] = a.y.w ? a.y.w[part] : 1.f;
        wt[k] = on ? wt[k] * a.mult : 0.f;
        #pragma unroll
        for (int i = 0; i < NV; ++i) {
          const int c = (i * TPR + tid) * VEC;
          t[k][i] = Held<F32, VEC>{};
          if (c < W && on) t[k][i].load(a.y.y, part * W + c);
        }
      }
    };
    if (n > 0) fetch(0);
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      h[i] = Pack<VEC>{};
      if (c < W) h[i] = ldv<true, VEC>(a.x, row * W + c);
    }
    also();
    for (int k0 = 0; k0 < n; k0 += CH) {
      if (k0) fetch(k0);
      #pragma unroll
      for (int k = 0; k < CH; ++k)
        #pragma unroll
        for (int i = 0; i < NV; ++i) {
          const Pack<VEC> u = t[k][i].up();
          #pragma unroll
          for (int j = 0; j < VEC; ++j) h[i].v[j] = fmaf(wt[k], u.v[j], h[i].v[j]);
        }
    }
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      if (c >= W) continue;
      if (a.add) {
        const Pack<VEC> e = ldv<true, VEC>(a.add, row * W + c);
        #pragma unroll
        for (int j = 0; j < VEC; ++j) h[i].v[j] += e.v[j];
      }
      if (a.step) {
        const Pack<VEC> e = ldv<F32, VEC>(a.step, c);
        #pragma unroll
        for (int j = 0; j < VEC; ++j) h[i].v[j] += e.v[j];
      }
      if (store) stv<true, VEC>(a.xo, row * W + c, h[i]);
    }
    layer_norm_rows<TPR, VEC, NV>(h, tid, W, a.eps, a.nxt.rms, red);
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      const Pack<VEC> w = wn[i].up();
      #pragma unroll
      for (int j = 0; j < VEC; ++j) h[i].v[j] *= w.v[j];
      if (a.nxt.b && c < W) {
        const Pack<VEC> b = ldv<F32, VEC>(a.nxt.b, c);
        #pragma unroll
        for (int j = 0; j < VEC; ++j) h[i].v[j] += b.v[j];
      }
    }
  };

  Pack<VEC> before[NV], h[NV];
  auto recall = [&](int row, int s) {
    const bool old = s >= 0 && r.pos[row] > 0;
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      before[i] = Pack<VEC>{};
      if (old && c < W) before[i] = ldv<true, VEC>(a.state, (long)s * W + c);
    }
  };
  auto keep = [&](int s) {
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      if (c < W) stv<true, VEC>(a.state, (long)s * W + c, h[i]);
    }
  };
  auto blend = [&](int row) {
    #pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int c = (i * TPR + tid) * VEC;
      const Pack<VEC> m = mix[i].up();
      Pack<VEC> o;
      #pragma unroll
      for (int j = 0; j < VEC; ++j) {
        o.v[j] = fmaf(before[i].v[j] - h[i].v[j], m.v[j], h[i].v[j]);
        before[i].v[j] = h[i].v[j];
      }
      if (c < W) stv<F32, VEC>(a.h, (long)row * W + c, o);
    }
  };
  if constexpr (!WALK) {
    const int s = a.shift ? r.slot[row0] : -1;
    make(row0, true, h, [&] { recall(row0, s); });
    if (s >= 0) keep(s);
    blend(row0);
  } else {
    // k -1: the row before the first, nothing but its norm.  A portion's last
    // row comes before its first one (`ahead`), for what the slot keeps.
    #pragma unroll
    for (int i = 0; i < NV; ++i) before[i] = Pack<VEC>{};
    bool ahead = false;
    int k = a.shift && !starts(r, row0) ? -1 : 0;
    while (k < rows) {
      const int row = row0 + k;
      int s = -1, at = row;
      if (k >= 0 && a.shift && starts(r, row)) {
        s = r.slot[row];
        if (!ahead) {
          recall(row, s);
          const int end = s >= 0 ? last_row(r, s) : -1;
          ahead = end >= 0;
          if (ahead) at = end;
        } else {
          ahead = false;
        }
      }
      make(at, k >= 0 && !ahead, h, [] {});
      if (ahead) {
        keep(s);
        continue;
      }
      if (k >= 0) {
        blend(row);
      } else {
        #pragma unroll
        for (int i = 0; i < NV; ++i) before[i] = h[i];
      }
      ++k;
    }
  }
}

template <bool F32, int VEC>
void launch_shift(const ShiftArgs& a, const RaggedRows& r, hipStream_t st) {
  // more rows a group: less work done twice; fewer: more groups
  const int rest = r.T - r.n_dec;
  const int per = !a.shift || rest <= 512 ? 1 : rest <= 2048 ? 2 : rest <= 4096 ? 4 : 8;
  const int tasks = (rest + per - 1) / per;
  #define SN_ONE(TPR, NV, WALK, N)                                             \
    if (N > 0)                                                                 \
      hipLaunchKernelGGL((shift_norm_kernel<F32, TPR, VEC, NV, WALK>),         \
                         dim3((unsigned)(((long)(N) * TPR + 255) / 256)),      \
                         dim3(256), 0, st, a, r, per)
  #define SN_GO(TPR, NV)                                                       \
    { SN_ONE(TPR, NV, false, r.n_dec); SN_ONE(TPR, NV, true, tasks); }
  if (a.W <= 64 * VEC) SN_GO(64, 1)
  else if (a.W <= 256 * VEC) SN_GO(256, 1)
  else if (a.W <= 512 * VEC) SN_GO(256, 2)
  else if (a.W <= 1024 * VEC) SN_GO(256, 4)
  else if (a.W <= 2048 * VEC) SN_GO(256, 8)
  else SN_GO(256, 16)             // up to 4096 * VEC (checked by the caller)
  #undef SN_GO
  #undef SN_ONE
}

}  // namespace

void lm_stream_embed(const EmbedArgs& a, const RaggedRows& r, bool f32,
                     hipStream_t st) {
  if (r.T <= 0) return;
  const bool v4 = a.W % 4 == 0;
  #define SE_GO(F, V)                                                          \
    hipLaunchKernelGGL((stream_embed_kernel<F, V>), dim3(r.T), dim3(256), 0, st, a, r)
  if (f32 && v4) SE_GO(true, 4);
  else if (f32) SE_GO(true, 1);
  else if (v4) SE_GO(false, 4);
  else SE_GO(false, 1);
  #undef SE_GO
}

void lm_shift_norm(const ShiftArgs& a, const RaggedRows& r, bool f32,
                   hipStream_t st) {
  if (r.T <= 0) return;
  const bool v4 = a.W % 4 == 0;
  if (f32) v4 ? launch_shift<true, 4>(a, r, st) : launch_shift<true, 1>(a, r, st);
  else v4 ? launch_shift<false, 4>(a, r, st) : launch_shift<false, 1>(a, r, st);
}
