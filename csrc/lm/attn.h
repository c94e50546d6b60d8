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

// A score times `scale` through the soft cap c tanh(x / c), in base 2, plus an
// addend.  Where every score of a wave is below 0.4 c (small(max |score|)) a
// polynomial in the square serves, four multiply-adds, relative error 1e-7
// (fitted to tanh(y) / y on [0, 0.4]); else c - 2 c / (exp(2 x / c) + 1).
struct SoftCap {
  float in, out, c2, limit;       // limit: of the polynomial, for a raw score
  float p0, p1, p2, p3;
  DEVINL SoftCap(const AttnArgs& a, float log2e) {
    const bool on = a.softcap > 0.f;
    const float r = on ? a.scale / a.softcap : 0.f, r2 = r * r;
    in = 2.f * log2e * r;
    out = a.softcap * log2e;
    c2 = -2.f * out;
    limit = on ? 0.4f / fabsf(r) : INFINITY;
    const float f = a.scale * log2e;          // no cap: this alone
    p0 = on ? f * 0.999999904f : f;
    p1 = -0.333313902f * f * r2;
    p2 = 0.132714383f * f * r2 * r2;
    p3 = -0.0475728106f * f * r2 * r2 * r2;
  }
  DEVINL bool small(float most) const { return !__any(most > limit); }
  DEVINL float near(float s, float b) const {
    const float t = s * s;
    return fmaf(s, fmaf(t, fmaf(t, fmaf(t, p3, p2), p1), p0), b);
  }
  DEVINL float any(float s, float b) const {
    const float e = __builtin_amdgcn_exp2f(s * in);
    return fmaf(c2, __builtin_amdgcn_rcpf(e + 1.f), out + b);
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
