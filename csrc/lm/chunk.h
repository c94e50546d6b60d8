// Building blocks of the recurrences that read prompts in tiles of 64
// tokens: staging rows, a tile's contribution to a state, a tile's queries
// against its incoming state.  States are kept transposed, [dv][dk].
#pragma once

#include "lm.h"
#include "tile.h"

// A tile's 64 x D elements, 8 at a time: load() has every load in flight
// together, put(j, c, raw) visits them; what lies past `rows` or `width` is
// zeros.
template <bool F32, int D> struct RowStage {
  static constexpr int N = LM_TILE * (D / 8) / 256;
  Raw8<F32> r[N];
  DEVINL void load(const typename Num<F32>::E* p0, long ld, int rows,
                   int width, bool aligned) {
    #pragma unroll
    for (int it = 0; it < N; ++it) {
      const int u = it * 256 + threadIdx.x, c = (u % (D / 8)) * 8;
      const typename Num<F32>::E* p = p0 + (long)min(u / (D / 8), rows - 1) * ld;
      if (aligned) r[it].load(p + (c < width ? c : 0), 8, true);
      else r[it].load(p + c, width - c, false);
    }
  }
  template <typename Put> DEVINL void visit(int rows, int width, Put put) {
    #pragma unroll
    for (int it = 0; it < N; ++it) {
      const int u = it * 256 + threadIdx.x;
      const int j = u / (D / 8), c = (u % (D / 8)) * 8;
      if (j >= rows || c >= width) r[it] = Raw8<F32>{};
      put(j, c, r[it]);
    }
  }
  // into an operand tile
  DEVINL void put(const ColTile<F32, D>& V, int rows, int width) {
    visit(rows, width, [&](int j, int c, const Raw8<F32>& x) {
      if constexpr (F32) V.put8(j, c, x.e);
      else V.put_raw(j, c, *(const bf16x8*)x.e);
    });
  }
};

// dst [dv][dk] = sum_j v_j k_j^T.  Wave w owns DV/4 state rows, in groups
// of 16; 64 columns at a time.
template <bool F32, int DK, int DV>
DEVINL void tile_outer(const ColTile<F32, DV>& V, const ColTile<F32, DK>& Kh,
                       const ColTile<F32, DK>& Kl, int dv, int dk,
                       float* __restrict__ dst) {
  using N = Num<F32>;
  const int w = threadIdx.x >> 6, l = threadIdx.x & 63;
  const int lr = l & 15, lg = l >> 4;
  constexpr int RT = DV / 64;
  for (int c4 = 0; c4 < DK / 16; c4 += 4) {
    if (c4 * 16 >= dk) break;
    f32x4 acc[RT][4];
    #pragma unroll
    for (int i = 0; i < RT; ++i)
      #pragma unroll
      for (int x = 0; x < 4; ++x) acc[i][x] = f32x4{0.f, 0.f, 0.f, 0.f};
    #pragma unroll
    for (int kb = 0; kb < LM_TILE / 32; ++kb) {
      typename N::Frag vf[4], kh[4], kl[4];
      // the wave's row tiles are among these four (RT divides 4)
      V.frags4((w * RT) / 4 * 4, kb, l, vf);
      Kh.frags4(c4, kb, l, kh);
      if constexpr (!F32) Kl.frags4(c4, kb, l, kl);
      #pragma unroll
      for (int i = 0; i < RT; ++i) {
        typename N::Frag r = vf[i];
        if constexpr (RT < 4) {
          // select tile w*RT + i without indexing registers by a variable
          #pragma unroll
          for (int y = 0; y < 4; ++y)
            if ((w * RT) % 4 + i == y) r = vf[y];
        }
        #pragma unroll
        for (int x = 0; x < 4; ++x) {
          if constexpr (!F32) acc[i][x] = N::mma(r, kl[x], acc[i][x]);
          acc[i][x] = N::mma(r, kh[x], acc[i][x]);
        }
      }
    }
    #pragma unroll
    for (int i = 0; i < RT; ++i)
      #pragma unroll
      for (int x = 0; x < 4; ++x)
        #pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = (w * RT + i) * 16 + 4 * lg + r;
          const int col = (c4 + x) * 16 + lr;
          if (row < dv && col < dk) dst[(long)row * dk + col] = acc[i][x][r];
        }
  }
}

// o[DV/16] of a wave's 16 rows = queries against the state S [dv][dk], 64
// state rows at a time through X ([64][LDK], split); mul(kb, s, acc) is the
// product with the wave's query fragment kb.
template <bool F32, int DK, int DV, int LDK, typename Mul>
DEVINL void times_state(const float* __restrict__ S, int dv, int dk,
                        const Split<F32>& X, f32x4 (&o)[DV / 16], Mul mul) {
  const int tid = threadIdx.x, l = tid & 63, lr = l & 15, lg = l >> 4;
  const bool s_al = dk % 8 == 0;
  #pragma unroll
  for (int vb = 0; vb < DV / 64; ++vb) {
    __syncthreads();
    constexpr int NS = 64 * (DK / 8) / 256;
    float v[NS][8];
    #pragma unroll
    for (int it = 0; it < NS; ++it) {
      const int u = it * 256 + tid, c = (u % (DK / 8)) * 8;
      const long row = min(vb * 64 + u / (DK / 8), dv - 1);
      if (s_al)                                // uniform
        load8<true>(S + row * dk + (c < dk ? c : 0), 8, true, v[it]);
      else
        load8<true>(S + row * dk + c, dk - c, false, v[it]);
    }
    #pragma unroll
    for (int it = 0; it < NS; ++it) {
      const int u = it * 256 + tid, j = u / (DK / 8), c = (u % (DK / 8)) * 8;
      const bool on = vb * 64 + j < dv && c < dk;
      #pragma unroll
      for (int i = 0; i < 8; ++i) v[it][i] = on ? v[it][i] : 0.f;
      X.put8(j * LDK + c, v[it]);
    }
    __syncthreads();
    #pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
      #pragma unroll
      for (int kb = 0; kb < DK / 32; ++kb)
        acc = mul(kb, X.load((i * 16 + lr) * LDK, kb * 32 + lg * 8), acc);
      o[vb * 4 + i] = acc;
    }
  }
}
