// What the attention kernels share beside tile.h.
#pragma once

#include "lm.h"
#include "tile.h"

// the sink's score of a head (a.has_sink)
template <bool F32>
DEVINL float sink_score(const AttnArgs& a, int h) {
  using E = typename Num<F32>::E;
  return a.sink ? Num<F32>::up(((const E*)a.sink)[h]) : a.sink0;
}

// what a query at position p is multiplied by
DEVINL float temperature(const AttnArgs& a, int p) {
  return a.t_every ? 1.0f + a.t_coef * logf((float)((p + 1) / a.t_every + 1))
                   : 1.0f;
}

// first position that the one at p sees through its chunk or window
DEVINL int first_seen(const AttnArgs& a, int p) {
  if (!a.size) return 0;
  return a.bias ? max(0, p - a.size + 1) : p - p % a.size;
}

// The pages that rows [p0, p1] see, in order: those of the kept first tokens
// that lie before the others, then the others.
struct PageList {
  int kept, first, n;
  DEVINL PageList(const AttnArgs& a, int p0, int p1) {
    first = first_seen(a, p0) / LM_PAGE;
    kept = min((a.keep + LM_PAGE - 1) / LM_PAGE, first);
    n = kept + p1 / LM_PAGE - first + 1;
  }
  DEVINL int operator[](int i) const { return i < kept ? i : first + i - kept; }
};

// A score times `scale` through the soft cap and to base 2, bias aside:
// c tanh(x / c) = c - 2 c / (exp(2 x / c) + 1).
struct SoftCap {
  float in, out, c2;     // exponent's factor, factors of the result
  bool on;
  DEVINL explicit SoftCap(const AttnArgs& a, float log2e) {
    on = a.softcap > 0.f;
    in = on ? 2.f * log2e * a.scale / a.softcap : 0.f;
    out = on ? a.softcap * log2e : a.scale * log2e;
    c2 = -2.f * out;
  }
  DEVINL float operator()(float s) const {
    if (!on) return s * out;
    return fmaf(c2, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * in) + 1.f), out);
  }
};

DEVINL float sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// Tied form: place of 8-column chunk cb of key j in a 64-key image of which
// rows are written or read 16 bytes a lane, and columns by transpose reads:
// four consecutive keys lie in different pairs of chunks, 8 (DK 64) or 16
// keys in different chunks.
template <int DK>
DEVINL int tied_chunk(int j, int cb) {
  if constexpr (DK == 64) return cb ^ (((j & 3) << 1) | ((j >> 2) & 1));
  else return cb ^ (((j & 7) << 1) | ((j >> 3) & 1));
}
