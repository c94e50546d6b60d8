// Gated linear attention: per head a float state S (kept transposed,
// [dv][dk]) whose columns, one per key channel, decay each by a factor of
// their own and of the token:
//     S_t = S_(t-1) diag(alpha_t) + v_t k_t^T      o_t = S_t q_t
// with log2 alpha = -log2(1 + exp(-z)) / tau, z = A2 u + b, and a per-head norm
// and a silu gate behind it.
//
// Prompts run in three launches over tiles of up to 64 tokens, as retention
// does: each tile's contribution to the state and its decay, the recurrence
// over a sequence's tiles, the outputs.  A decay spans many powers of two and
// cannot be divided out, so a tile is four sub-tiles of 16 tokens, and only
// differences that are never positive are raised: with F_i the log decay from
// the start of i's sub-tile up to i and T_s that of all of sub-tile s,
//   k^_j = k_j 2^(T_s - F_j)            what reaches the end of j's sub-tile
//   q_i 2^(F_i)                         against k^ of the sub-tile before,
//   q_i 2^(F_i + T_(s-1))               of the one before that, and so on; the
//                                       last of these meets the incoming state.
// Inside a sub-tile q_i 2^(F_i - T_s) against k^ is right as long as T_s is
// above -LIMIT; a sub-tile that decays more than that takes its 16 x 16 scores
// one by one.
//
// The projections enter as they are; decays, weighted q and k, scores and the
// state are float (in bf16 mode the matrix products take them as two bf16
// parts, see tile.h).

#include "chunk.h"

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr float LIMIT = 60.f;

DEVINL float pow2(float x) { return __builtin_amdgcn_exp2f(x); }
DEVINL float silu(float z) { return z / (1.0f + expf(-z)); }

// log2 of a channel's decay.  log(1 + t) as log(u) t / (u - 1), u the rounded
// 1 + t: the rounding of u cancels (Higham, "Accuracy and Stability of
// Numerical Algorithms").
template <bool F32>
DEVINL float log_decay(const GlaArgs& a, float z) {
  if constexpr (F32)
    return -(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)))) * (LOG2E * a.inv_tau);
  const float t = pow2(-fabsf(z) * LOG2E), u = 1.f + t;
  const float l = u == 1.f ? t * LOG2E
                           : __builtin_amdgcn_logf(u) * t * __builtin_amdgcn_rcpf(u - 1.f);
  return -fmaf(fmaxf(-z, 0.f), LOG2E, l) * a.inv_tau;
}

// Log decays of a tile: F [64][DK] from the start of a token's sub-tile up to
// it, tot [4][DK] those of whole sub-tiles.  Wave w has sub-tile w, eight
// 16-channel tiles at a time; the first 32 columns of the sum over the rank
// (all of them, as a rule) have their loads in flight together.
template <bool F32, int DK>
DEVINL void tile_decays(const GlaArgs& a, int row0, int rows, int h, float* F,
                        float* tot) {
  using N = Num<F32>;
  using E = typename N::E;
  constexpr int CT = DK / 16 < 8 ? DK / 16 : 8;
  const int w = threadIdx.x >> 6, l = threadIdx.x & 63;
  const int lr = l & 15, lg = l >> 4;
  const bool al = a.rank % 8 == 0, u_al = al && a.dk % 8 == 0 && a.dv % 8 == 0;
  const E* u = (const E*)a.u + (long)(row0 + min(16 * w + lr, rows - 1)) * a.ld;
  const E* m0 = (const E*)a.a2 + (long)h * a.dk * a.rank;
  Raw8<F32> x;
  x.load(u + 8 * lg, a.rank - 8 * lg, u_al);
  for (int c0 = 0; c0 < a.dk; c0 += 16 * CT) {
    Raw8<F32> y[CT];
    E b[CT];
    #pragma unroll
    for (int i = 0; i < CT; ++i) {
      const int c = min(c0 + i * 16 + lr, a.dk - 1);
      y[i].load(m0 + (long)c * a.rank + 8 * lg, a.rank - 8 * lg, al);
      b[i] = ((const E*)a.a2b)[(long)h * a.dk + c];
    }
    f32x4 z[CT];
    #pragma unroll
    for (int i = 0; i < CT; ++i)
      z[i] = N::mma(N::load(x.e, 0), N::load(y[i].e, 0), f32x4{0.f, 0.f, 0.f, 0.f});
    for (int k = 32 + 8 * lg; k - 8 * lg < a.rank; k += 32) {
      Raw8<F32> v;
      v.load(u + k, a.rank - k, u_al);
      #pragma unroll
      for (int i = 0; i < CT; ++i) {
        y[i].load(m0 + (long)min(c0 + i * 16 + lr, a.dk - 1) * a.rank + k,
                  a.rank - k, al);
        z[i] = N::mma(N::load(v.e, 0), N::load(y[i].e, 0), z[i]);
      }
    }
    #pragma unroll
    for (int i = 0; i < CT; ++i) {
      if (c0 + i * 16 >= a.dk) continue;      // uniform
      float f[4], s = 0.f;
      #pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float d = log_decay<F32>(a, z[i][r] + N::up(b[i]));
        s += 16 * w + 4 * lg + r < rows ? d : 0.f;
        f[r] = s;
      }
      // tokens 4 lg .. of the sub-tile: add what the lane groups before have
      float before = 0.f;
      #pragma unroll
      for (int g = 0; g < 3; ++g) {
        const float o = __shfl(s, g * 16 + lr, 64);
        before += g < lg ? o : 0.f;
      }
      #pragma unroll
      for (int r = 0; r < 4; ++r) {
        f[r] += before;
        F[(16 * w + 4 * lg + r) * DK + c0 + i * 16 + lr] = f[r];
      }
      if (lg == 3) tot[w * DK + c0 + i * 16 + lr] = f[3];
    }
  }
}

DEVINL bool gla_aligned(const GlaArgs& a) { return a.dk % 8 == 0 && a.dv % 8 == 0; }

// contribution of one tile and head to the state, and its channels' decays
template <bool F32, int DK, int DV>
__global__ void __launch_bounds__(256, !F32 && DK <= 128 && DV <= 128 ? 3 : 1)
gla_chunk_state_kernel(GlaArgs a, const int4* __restrict__ tiles,
                       float* __restrict__ cs, float* __restrict__ cd) {
  using E = typename Num<F32>::E;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ float tot[4 * DK], tail[4 * DK];
  float* F = (float*)smem;                    // first F, then the operands
  const ColTile<F32, DK> Kh{(E*)smem}, Kl{Kh.p + Kh.SIZE};
  const ColTile<F32, DV> V{Kh.p + (F32 ? 1 : 2) * Kh.SIZE};

  const int4 t = tiles[blockIdx.y];
  const int h = blockIdx.x;
  const bool aligned = gla_aligned(a);
  const long cell = (long)blockIdx.y * a.H + h;
  RowStage<F32, DK> ks;
  RowStage<F32, DV> vs;
  ks.load((const E*)a.k + (long)t.x * a.ld + (long)h * a.dk, a.ld, t.y, a.dk,
          aligned);
  vs.load((const E*)a.v + (long)t.x * a.ld + (long)h * a.dv, a.ld, t.y, a.dv,
          aligned);
  tile_decays<F32, DK>(a, t.x, t.y, h, F, tot);
  __syncthreads();
  for (int c = threadIdx.x; c < a.dk; c += 256) {
    float s = 0.f;                            // what follows each sub-tile
    #pragma unroll
    for (int i = 3; i >= 0; --i) {
      tail[i * DK + c] = s;
      s += tot[i * DK + c];
    }
    cd[cell * a.dk + c] = pow2(s);
  }
  __syncthreads();
  float wk[RowStage<F32, DK>::N][8];          // weighted keys
  int n = 0;
  ks.visit(t.y, a.dk, [&](int j, int c, const Raw8<F32>& x) {
    const float* f = F + j * DK + c;
    const int sub = (j >> 4) * DK + c;
    #pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float d = pow2((tot[sub + i] - f[i]) + tail[sub + i]);
      wk[n][i] = c + i < a.dk ? x[i] * d : 0.f;
    }
    ++n;
  });
  __syncthreads();                            // F is done with
  n = 0;
  ks.visit(t.y, a.dk, [&](int j, int c, const Raw8<F32>&) {
    Kh.put8(j, c, wk[n]);
    if constexpr (!F32) {
      #pragma unroll
      for (int i = 0; i < 8; ++i) wk[n][i] -= bf2f(cvt_bf16(wk[n][i]));
      Kl.put8(j, c, wk[n]);
    }
    ++n;
  });
  vs.put(V, t.y, a.dv);
  __syncthreads();
  tile_outer<F32, DK, DV>(V, Kh, Kl, a.dv, a.dk, cs + cell * a.dv * a.dk);
}

// S <- S diag(d) + contribution over a sequence's tiles; leaves every tile's
// incoming state in the scratch and the final one in the slot.  A sequence's
// first tokens (position 0) start from zero whatever the slot held before.
__global__ void __launch_bounds__(256)
gla_scan_kernel(GlaArgs a, const int4* __restrict__ seqs, float* __restrict__ cs,
                const float* __restrict__ cd) {
  const int4 q = seqs[blockIdx.z];          // first tile, tiles, pos0, slot
  const int h = blockIdx.y;
  const long n = (long)a.dv * a.dk;
  const long e = (long)blockIdx.x * 256 + threadIdx.x;
  if (e >= n) return;
  float* st = a.state + ((long)q.w * a.H + h) * n + e;
  float s = q.z == 0 ? 0.f : *st;
  float* p = cs + ((long)q.x * a.H + h) * n + e;
  const float* d = cd + ((long)q.x * a.H + h) * a.dk + e % a.dk;
  const long step = (long)a.H * n, dstep = (long)a.H * a.dk;
  float pn = *p, dn = *d;
  for (int c = 0; c < q.y; ++c) {
    const float add = pn, keep = dn;
    if (c + 1 < q.y) {
      pn = p[step];
      d += dstep;
      dn = *d;
    }
    *p = s;
    s = fmaf(s, keep, add);
    p += step;
  }
  *st = s;
}

template <bool F32, int DK, int DV>
__global__ void __launch_bounds__(256)
gla_chunk_out_kernel(GlaArgs a, const int4* __restrict__ tiles,
                     const float* __restrict__ cs) {
  using N = Num<F32>;
  using E = typename N::E;
  using S = Split<F32>;
  constexpr int LDK = DK + N::PAD, LDJ = LM_TILE + N::PAD, KB = DK / 32;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __shared__ float tot[4 * DK];
  E* Xb = (E*)smem;                         // [PARTS][64][LDK]: k^, then S
  E* rest = Xb + S::PARTS * LM_TILE * LDK;  // first F, then scores and values
  float* F = (float*)rest;
  const S X{Xb, Xb + LM_TILE * LDK};
  const S P{rest, rest + LM_TILE * LDJ};
  const ColTile<F32, DV> V{rest + S::PARTS * LM_TILE * LDJ};

  const int4 t = tiles[blockIdx.y];
  const int h = blockIdx.x;
  const int tid = threadIdx.x, w = tid >> 6, l = tid & 63;
  const int lr = l & 15, lg = l >> 4;
  const bool aligned = gla_aligned(a);
  const long cell = (long)blockIdx.y * a.H + h;

  RowStage<F32, DK> ks;
  RowStage<F32, DV> vs;
  Raw8<F32> qr[KB];                         // this wave's 16 queries
  const E* k0 = (const E*)a.k + (long)t.x * a.ld + (long)h * a.dk;
  const E* q0 = (const E*)a.q + (long)(t.x + min(16 * w + lr, t.y - 1)) * a.ld +
                (long)h * a.dk;
  ks.load(k0, a.ld, t.y, a.dk, aligned);
  vs.load((const E*)a.v + (long)t.x * a.ld + (long)h * a.dv, a.ld, t.y, a.dv,
          aligned);
  #pragma unroll
  for (int kb = 0; kb < KB; ++kb) {
    const int c = kb * 32 + lg * 8;
    if (aligned) qr[kb].load(q0 + (c < a.dk ? c : 0), 8, true);
    else qr[kb].load(q0 + c, a.dk - c, false);
  }
  tile_decays<F32, DK>(a, t.x, t.y, h, F, tot);
  __syncthreads();

  ks.visit(t.y, a.dk, [&](int j, int c, const Raw8<F32>& x) {
    float v[8];
    const float* f = F + j * DK + c;
    const int sub = (j >> 4) * DK + c;
    #pragma unroll
    for (int i = 0; i < 8; ++i)
      v[i] = c + i < a.dk ? x[i] * pow2(tot[sub + i] - f[i]) : 0.f;
    X.put8(j * LDK + c, v);
  });

  // q 2^F of this wave's rows; steep: a channel decays too far to divide by
  float qd[KB][8];
  bool steep = false;
  auto frag = [&](int kb, const float (&v)[8]) {
    typename S::Frag f;
    if constexpr (F32) {
      #pragma unroll
      for (int i = 0; i < 8; ++i) f.hi.v[i] = v[i];
    } else {
      #pragma unroll
      for (int i = 0; i < 8; ++i) {
        f.hi[i] = cvt_bf16(v[i]);
        f.lo[i] = cvt_bf16(v[i] - bf2f(f.hi[i]));
      }
    }
    return f;
  };
  typename S::Frag qs[KB];
  #pragma unroll
  for (int kb = 0; kb < KB; ++kb) {
    const int c = kb * 32 + lg * 8;
    float qi[8];
    #pragma unroll
    for (int i = 0; i < 8; ++i) {
      const bool on = c + i < a.dk;
      const float f = on ? F[(16 * w + lr) * DK + c + i] : 0.f;
      const float d = on ? tot[w * DK + c + i] : 0.f;
      const float q = on ? qr[kb][i] * a.qscale : 0.f;
      steep |= d < -LIMIT;
      qd[kb][i] = q * pow2(f);
      qi[i] = q * pow2(fminf(f - d, LIMIT));
    }
    qs[kb] = frag(kb, qi);
  }
  steep = __any(steep);
  __syncthreads();                          // k^ is there

  f32x4 sc[4];                              // scores against sub-tile ct
  #pragma unroll
  for (int ct = 0; ct < 4; ++ct) sc[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto against = [&](int ct) {              // of the queries in qs
    f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
    #pragma unroll
    for (int kb = 0; kb < KB; ++kb)
      s = mma_ss<F32>(qs[kb], X.load((ct * 16 + lr) * LDK, kb * 32 + lg * 8), s);
    return s;
  };
  f32x4 own;
  if (!steep) {
    own = against(w);
  } else {                                  // key j = lr, queries 4 lg + r
    own = f32x4{0.f, 0.f, 0.f, 0.f};
    const int jr = min(16 * w + lr, t.y - 1);
    const E* kj = k0 + (long)jr * a.ld;
    const float* Fj = F + (16 * w + lr) * DK;
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * w + 4 * lg + r;
      const E* qi = (const E*)a.q + (long)(t.x + min(i, t.y - 1)) * a.ld + (long)h * a.dk;
      float s = 0.f;
      if (lr <= 4 * lg + r)
        for (int c = 0; c < a.dk; ++c)
          s = fmaf(N::up(qi[c]) * a.qscale * N::up(kj[c]),
                   pow2(F[i * DK + c] - Fj[c]), s);
      own[r] = s;
    }
  }
  // back through the sub-tiles before; afterwards qd is what meets the state
  #pragma unroll
  for (int b = 3; b >= 0; --b) {
    if (b > w) continue;
    #pragma unroll
    for (int kb = 0; kb < KB; ++kb) {
      if (b < w) {
        const int c = kb * 32 + lg * 8;
        qs[kb] = frag(kb, qd[kb]);
        #pragma unroll
        for (int i = 0; i < 8; ++i)
          qd[kb][i] *= c + i < a.dk ? pow2(tot[b * DK + c + i]) : 0.f;
      }
    }
    if (b < w) sc[b] = against(b);
  }
  #pragma unroll
  for (int kb = 0; kb < KB; ++kb) qs[kb] = frag(kb, qd[kb]);
  __syncthreads();                          // F and k^ are done with
  vs.put(V, t.y, a.dv);
  #pragma unroll
  for (int ct = 0; ct < 4; ++ct)
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 4 * lg + r;
      float s = sc[ct][r];
      if (ct == w) s = lr <= i ? own[r] : 0.f;
      P.put((16 * w + i) * LDJ + ct * 16 + lr, s);
    }

  f32x4 o[DV / 16];                         // against the incoming state
  times_state<F32, DK, DV, LDK>(
      cs + cell * a.dv * a.dk, a.dv, a.dk, X, o,
      [&](int kb, const typename S::Frag& s, f32x4 acc) {
        return mma_ss<F32>(qs[kb], s, acc);
      });
  // gates: all in flight here, used in the epilogue
  E gz[4][DV / 16];
  float nw[DV / 16];
  #pragma unroll
  for (int i = 0; i < DV / 16; ++i)
    nw[i] = N::up(((const E*)a.norm)[min(i * 16 + lr, a.dv - 1)]) * a.out_scale;
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    const E* gate = (const E*)a.gate +
                    (long)(t.x + min(16 * w + 4 * lg + r, t.y - 1)) * a.ld +
                    (long)h * a.dv;
    #pragma unroll
    for (int i = 0; i < DV / 16; ++i)
      gz[r][i] = gate[min(i * 16 + lr, a.dv - 1)];
  }
  #pragma unroll
  for (int kb = 0; kb < LM_TILE / 32; ++kb) {
    if (kb * 2 > w) continue;               // keys after all of these rows
    const auto pf = P.load((16 * w + lr) * LDJ, kb * 32 + lg * 8);
    #pragma unroll
    for (int i = 0; i < DV / 16; i += 4) {
      typename N::Frag vf[4];
      V.frags4(i, kb, l, vf);
      #pragma unroll
      for (int x = 0; x < 4; ++x) o[i + x] = mma_sp<F32>(pf, vf[x], o[i + x]);
    }
  }
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    float ss = 0.f;
    #pragma unroll
    for (int i = 0; i < DV / 16; ++i) ss += o[i][r] * o[i][r];
    const float inv = 1.0f / sqrtf(sum16(ss) / (float)a.dv + a.eps);
    const int row = 16 * w + 4 * lg + r;
    if (row >= t.y) continue;
    E* dst = (E*)a.out + (long)(t.x + row) * a.ldo + (long)h * a.dv;
    #pragma unroll
    for (int i = 0; i < DV / 16; ++i) {
      const int c = i * 16 + lr;
      if (c < a.dv) dst[c] = N::down(o[i][r] * inv * nw[i] * silu(N::up(gz[r][i])));
    }
  }
}

// One token of one row and head per block.
template <bool F32, int NT>
__global__ void __launch_bounds__(NT)
gla_decode_kernel(GlaArgs a, const int* __restrict__ pos,
                  const int* __restrict__ slot) {
  using N = Num<F32>;
  using E = typename N::E;
  __shared__ __attribute__((aligned(16))) float q_s[256], k_s[256], d_s[256];
  __shared__ float o_s[256], red[NT / 64];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x;
  E* dst = (E*)a.out + (long)row * a.ldo + (long)h * a.dv;
  const int s = slot[row];
  if (s < 0) {
    for (int c = tid; c < a.dv; c += NT) dst[c] = N::down(0.f);
    return;
  }
  const bool fresh = pos[row] == 0;
  const long at = (long)row * a.ld;
  const E* vrow = (const E*)a.v + at + (long)h * a.dv;
  const E* grow = (const E*)a.gate + at + (long)h * a.dv;
  const E* u = (const E*)a.u + at;
  // decays, the sum over the rank spread over 4 lanes a channel
  for (int c0 = 0; c0 < a.dk; c0 += NT / 4) {
    const int c = c0 + tid / 4;
    float z = 0.f;
    if (c < a.dk) {
      const E* m = (const E*)a.a2 + ((long)h * a.dk + c) * a.rank;
      for (int k = tid & 3; k < a.rank; k += 4) z = fmaf(N::up(m[k]), N::up(u[k]), z);
    }
    z = group_sum<4>(z);
    if (c < a.dk && (tid & 3) == 0)
      d_s[c] = pow2(log_decay<F32>(
          a, z + N::up(((const E*)a.a2b)[(long)h * a.dk + c])));
  }
  for (int c = tid; c < a.dk; c += NT) {
    q_s[c] = N::up(((const E*)a.q)[at + (long)h * a.dk + c]) * a.qscale;
    k_s[c] = N::up(((const E*)a.k)[at + (long)h * a.dk + c]);
  }
  __syncthreads();

  float* S = a.state + ((long)s * a.H + h) * a.dv * a.dk;
  if (a.dk % 4 == 0) {
    int lpr = 1;                            // lanes that share a state row
    while (lpr * 4 < a.dk) lpr <<= 1;
    const int c = (tid & (lpr - 1)) * 4;
    const int rstep = NT / lpr;
    constexpr int RB = 4;
    const bool in = c < a.dk;
    f32x4 kv = f32x4{0.f, 0.f, 0.f, 0.f}, qv = kv, dv = kv;
    if (in) {
      kv = *(const f32x4*)(k_s + c);
      qv = *(const f32x4*)(q_s + c);
      dv = *(const f32x4*)(d_s + c);
    }
    for (int r0 = tid / lpr; r0 < a.dv; r0 += rstep * RB) {
      f32x4 x[RB];
      #pragma unroll
      for (int i = 0; i < RB; ++i) {
        const int r = r0 + i * rstep;
        x[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (in && r < a.dv && !fresh) x[i] = *(const f32x4*)(S + (long)r * a.dk + c);
      }
      #pragma unroll
      for (int i = 0; i < RB; ++i) {
        const int r = r0 + i * rstep;
        float d = 0.f;
        if (in && r < a.dv) {
          const float v = N::up(vrow[r]);
          #pragma unroll
          for (int j = 0; j < 4; ++j) {
            x[i][j] = fmaf(x[i][j], dv[j], kv[j] * v);
            d = fmaf(x[i][j], qv[j], d);
          }
          *(f32x4*)(S + (long)r * a.dk + c) = x[i];
        }
        for (int o = 1; o < lpr; o <<= 1) d += __shfl_xor(d, o, 64);
        if (c == 0 && r < a.dv) o_s[r] = d;
      }
    }
  } else {
    const int w = tid >> 6, l = tid & 63;
    for (int r = w; r < a.dv; r += NT / 64) {
      const float v = N::up(vrow[r]);
      float d = 0.f;
      for (int c = l; c < a.dk; c += 64) {
        float* e = S + (long)r * a.dk + c;
        const float x = fmaf(fresh ? 0.f : *e, d_s[c], k_s[c] * v);
        *e = x;
        d = fmaf(x, q_s[c], d);
      }
      d = wave_reduce_sum(d);
      if (l == 0) o_s[r] = d;
    }
  }
  __syncthreads();
  float qd = 0.f;
  for (int c = tid; c < a.dv; c += NT) qd += o_s[c] * o_s[c];
  qd = wave_reduce_sum(qd);
  if ((tid & 63) == 0) red[tid >> 6] = qd;
  __syncthreads();
  float all = 0.f;
  #pragma unroll
  for (int i = 0; i < NT / 64; ++i) all += red[i];
  const float inv = a.out_scale / sqrtf(all / (float)a.dv + a.eps);
  for (int c = tid; c < a.dv; c += NT)
    dst[c] = N::down(o_s[c] * inv * N::up(((const E*)a.norm)[c]) *
                     silu(N::up(grow[c])));
}

template <bool F32, int DK, int DV>
void launch_prefill(const GlaArgs& a, const int4* tiles, int n_tiles,
                    const int4* seqs, int n_seqs, float* ws, hipStream_t st) {
  using N = Num<F32>;
  using S = Split<F32>;
  using V = ColTile<F32, DV>;
  constexpr size_t es = sizeof(typename N::E);
  constexpr int LDJ = LM_TILE + N::PAD;
  constexpr size_t f = sizeof(float) * LM_TILE * DK;
  constexpr size_t lds1 =
      std::max(f, es * (S::PARTS * ColTile<F32, DK>::SIZE + V::SIZE));
  constexpr size_t lds2 =
      es * S::PARTS * LM_TILE * (DK + N::PAD) +
      std::max(f, es * (S::PARTS * LM_TILE * LDJ + V::SIZE));
  constexpr size_t fixed = sizeof(float) * 8 * DK;     // tot, tail
  static_assert(lds1 + fixed <= 160 * 1024 && lds2 + fixed <= 160 * 1024,
                "exceeds the CU's LDS");
  static const hipError_t attr1 = hipFuncSetAttribute(
      (const void*)gla_chunk_state_kernel<F32, DK, DV>,
      hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds1);
  static const hipError_t attr2 = hipFuncSetAttribute(
      (const void*)gla_chunk_out_kernel<F32, DK, DV>,
      hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds2);
  (void)attr1;
  (void)attr2;
  float* cs = ws;
  float* cd = cs + (long)n_tiles * a.H * a.dv * a.dk;
  hipLaunchKernelGGL((gla_chunk_state_kernel<F32, DK, DV>), dim3(a.H, n_tiles),
                     dim3(256), lds1, st, a, tiles, cs, cd);
  hipLaunchKernelGGL(gla_scan_kernel,
                     dim3((unsigned)(((long)a.dv * a.dk + 255) / 256), a.H, n_seqs),
                     dim3(256), 0, st, a, seqs, cs, (const float*)cd);
  hipLaunchKernelGGL((gla_chunk_out_kernel<F32, DK, DV>), dim3(a.H, n_tiles),
                     dim3(256), lds2, st, a, tiles, (const float*)cs);
}

template <bool F32, int DK>
void pick_dv(const GlaArgs& a, const int4* tiles, int nt, const int4* seqs,
             int ns, float* ws, hipStream_t st) {
  if (a.dv <= 64) launch_prefill<F32, DK, 64>(a, tiles, nt, seqs, ns, ws, st);
  else if (a.dv <= 128) launch_prefill<F32, DK, 128>(a, tiles, nt, seqs, ns, ws, st);
  else launch_prefill<F32, DK, 256>(a, tiles, nt, seqs, ns, ws, st);
}

template <bool F32>
void pick_dk(const GlaArgs& a, const int4* tiles, int nt, const int4* seqs,
             int ns, float* ws, hipStream_t st) {
  if (a.dk <= 64) pick_dv<F32, 64>(a, tiles, nt, seqs, ns, ws, st);
  else if (a.dk <= 128) pick_dv<F32, 128>(a, tiles, nt, seqs, ns, ws, st);
  else pick_dv<F32, 256>(a, tiles, nt, seqs, ns, ws, st);
}

template <bool F32>
void run_decode(const GlaArgs& a, const int* pos, const int* slot, int R,
                hipStream_t st) {
  // every thread keeps 4 state vectors (16 floats) in flight
  const int need = a.dk * a.dv / 16;
  #define GL_GO(NT)                                                            \
    hipLaunchKernelGGL((gla_decode_kernel<F32, NT>), dim3(a.H, R), dim3(NT), 0, \
                       st, a, pos, slot)
  if (need <= 256) GL_GO(256);
  else if (need <= 512) GL_GO(512);
  else GL_GO(1024);
  #undef GL_GO
}

}  // namespace

long lm_gla_scratch(const GlaArgs& a, int n_tiles) {
  return (long)n_tiles * a.H * a.dk * (a.dv + 1);
}

void lm_gla_prefill(const GlaArgs& a, const int4* tiles, int n_tiles,
                    const int4* seqs, int n_seqs, float* ws, bool f32,
                    hipStream_t stream) {
  if (n_tiles <= 0) return;
  if (f32) pick_dk<true>(a, tiles, n_tiles, seqs, n_seqs, ws, stream);
  else pick_dk<false>(a, tiles, n_tiles, seqs, n_seqs, ws, stream);
}

void lm_gla_decode(const GlaArgs& a, const int* pos, const int* slot, int R,
                   bool f32, hipStream_t stream) {
  if (R <= 0) return;
  if (f32) run_decode<true>(a, pos, slot, R, stream);
  else run_decode<false>(a, pos, slot, R, stream);
}
