// Retention: per head a float state S (kept transposed, [dv][dk]) that
// decays by a constant each token and takes k v^T; o = S^T q, normed per
// head, gated by silu and handed to the output projection.
//
// Prompts run in three launches over tiles of up to 64 tokens:
//   chunk_state  every tile's own contribution to the state, in parallel
//   scan         the recurrence over a sequence's tiles, elementwise; leaves
//                each tile's incoming state in the scratch buffer and the
//                final one in the cache slot
//   chunk_out    o_i = d^(i+1) S_in^T q_i + sum_{j<=i} d^(i-j) (q_i.k_j) v_j,
//                the head norm and the gate in the epilogue
// A single new token (decode) is one launch that reads and writes the state
// once and does everything from the rotation to the gate.
//
// q and k are rotated while they are staged; from there on they, the decay
// powers and the state are float (in bf16 mode the matrix products take
// them as two bf16 parts, see tile.h).
//
// Linear attention with the same recurrence is served as well: silu of q, k
// and v as they are read (v is rounded to the model's type after it), and raw
// outputs for a norm over all heads.

#include "chunk.h"

namespace {

DEVINL float silu(float z) { return z / (1.0f + expf(-z)); }

// Rotated q or k elements c..c+7 of one head, times `mul`.  Element i of
// the first half of the rotated span pairs with i + rd/2.
template <bool F32>
DEVINL void load_rot8(const typename Num<F32>::E* head, int c, const RetArgs& a,
                      int pos, float mul, bool aligned, float* out) {
  load8<F32>(head + c, a.dk - c, aligned, out);
  const int half = a.rd >> 1;
  if (c < a.rd) {
    const float* ct = a.cos_t + (long)pos * half;
    const float* st = a.sin_t + (long)pos * half;
    if (aligned && half % 8 == 0) {          // the 8 lie in one half
      const bool low = c < half;
      const int i = low ? c : c - half;
      float o[8], cv[8], sv[8];
      load8<F32>(head + (low ? c + half : c - half), 8, true, o);
      load8<true>(ct + i, 8, true, cv);
      load8<true>(st + i, 8, true, sv);
      #pragma unroll
      for (int j = 0; j < 8; ++j)
        out[j] = low ? out[j] * cv[j] - o[j] * sv[j]
                     : out[j] * cv[j] + o[j] * sv[j];
    } else {
      #pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int e = c + j;
        if (e < a.rd) {
          const bool low = e < half;
          const int i = low ? e : e - half;
          const float o = Num<F32>::up(head[low ? e + half : e - half]);
          out[j] = low ? out[j] * ct[i] - o * st[i] : out[j] * ct[i] + o * st[i];
        }
      }
    }
  }
  if (a.silu) {
    #pragma unroll
    for (int j = 0; j < 8; ++j) out[j] = silu(out[j]);
  }
  #pragma unroll
  for (int j = 0; j < 8; ++j) out[j] *= mul;
}

// Visit a tile's 64 x D elements of one head's q or k, rotated and scaled by
// mul(j), 8 at a time: put(j, c, v).  Rows past `rows` are zeros.  The usual
// shapes take a branch-free path whose loads are all in flight together.
template <bool F32, int D, typename Mul, typename Put>
DEVINL void stage_rot(const typename Num<F32>::E* head0, const RetArgs& a,
                      int pos0, int rows, bool aligned, Mul mul, Put put) {
  constexpr int N = 64 * (D / 8) / 256;
  const int half = a.rd >> 1;
  if (aligned && half % 8 == 0) {
    Raw8<F32> own[N], oth[N];
    float cv[N][8], sv[N][8];
    #pragma unroll
    for (int it = 0; it < N; ++it) {
      const int u = it * 256 + threadIdx.x;
      const int j = min(u / (D / 8), rows - 1);
      int c = (u % (D / 8)) * 8;
      c = c < a.dk ? c : 0;
      const bool in = c < a.rd, low = c < half;
      const int oc = in ? (low ? c + half : c - half) : c;
      const typename Num<F32>::E* p = head0 + (long)j * a.ld;
      own[it].load(p + c, 8, true);
      oth[it].load(p + oc, 8, true);
      if (half) {                              // uniform
        const long ti = (long)(pos0 + j) * half + (in ? (low ? c : c - half) : 0);
        load8<true>(a.cos_t + ti, 8, true, cv[it]);
        load8<true>(a.sin_t + ti, 8, true, sv[it]);
      }
    }
    #pragma unroll
    for (int it = 0; it < N; ++it) {
      const int u = it * 256 + threadIdx.x;
      const int j = u / (D / 8), c = (u % (D / 8)) * 8;
      const bool in = c < a.rd, low = c < half;
      const float f = j < rows && c < a.dk ? mul(min(j, rows - 1)) : 0.f;
      float v[8];
      #pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float x = own[it][i], y = oth[it][i];
        float r = x;
        if (half) {
          const float w = low ? -y : y;
          r = in ? x * cv[it][i] + w * sv[it][i] : x;
        }
        v[i] = (a.silu ? silu(r) : r) * f;
      }
      put(j, c, v);
    }
  } else {
    for (int u = threadIdx.x; u < 64 * (D / 8); u += 256) {
      const int j = u / (D / 8), c = (u % (D / 8)) * 8;
      float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      if (j < rows)
        load_rot8<F32>(head0 + (long)j * a.ld, c, a, pos0 + j, mul(j), aligned, v);
      put(j, c, v);
    }
  }
}

// value rows of a tile
template <bool F32, int DV>
DEVINL void ret_values(const ColTile<F32, DV>& V, const typename Num<F32>::E* v0,
                       const RetArgs& a, int rows, bool aligned) {
  RowStage<F32, DV> r;
  r.load(v0, a.ld, rows, a.dv, aligned);
  if (!a.silu) return r.put(V, rows, a.dv);
  r.visit(rows, a.dv, [&](int j, int c, const Raw8<F32>& x) {
    float v[8];
    #pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = silu(x[i]);
    V.put8(j, c, v);
  });
}

DEVINL bool ret_aligned(const RetArgs& a) {
  return a.dk % 8 == 0 && a.dv % 8 == 0;
}

// state contribution of one tile and head: sum_j d^(n-1-j) v_j k_j^T
template <bool F32, int DK, int DV>
__global__ void __launch_bounds__(256)
ret_chunk_state_kernel(RetArgs a, const int4* __restrict__ tiles,
                       float* __restrict__ cs) {
  using E = typename Num<F32>::E;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const ColTile<F32, DV> V{(E*)smem};
  const ColTile<F32, DK> Kh{V.p + V.SIZE}, Kl{Kh.p + Kh.SIZE};

  const int4 t = tiles[blockIdx.y];
  const int h = blockIdx.x;   // heads of a row run together: whole rows stream
  const bool aligned = ret_aligned(a);
  const float* pw = a.pows + (long)h * (LM_TILE + 1);
  const E* base = (const E*)a.qkvg + (long)t.x * a.ld;

  stage_rot<F32, DK>(
      base + (long)(a.H + h) * a.dk, a, t.z, t.y, aligned,
      [&](int j) { return a.kscale * pw[t.y - 1 - j]; },
      [&](int j, int c, float* v) {
        Kh.put8(j, c, v);
        if constexpr (!F32) {
          #pragma unroll
          for (int i = 0; i < 8; ++i) v[i] -= bf2f(cvt_bf16(v[i]));
          Kl.put8(j, c, v);
        }
      });
  ret_values<F32, DV>(V, base + (long)2 * a.H * a.dk + (long)h * a.dv, a, t.y,
                      aligned);
  __syncthreads();

  tile_outer<F32, DK, DV>(V, Kh, Kl, a.dv, a.dk,
                          cs + ((long)blockIdx.y * a.H + h) * a.dv * a.dk);
}

// S <- d^n S + contribution over a sequence's tiles; a sequence's first
// tokens (position 0) start from zero whatever the slot held before.
__global__ void __launch_bounds__(256)
ret_scan_kernel(RetArgs a, const int4* __restrict__ tiles,
                const int4* __restrict__ seqs, float* __restrict__ cs) {
  const int4 q = seqs[blockIdx.z];          // first tile, tiles, pos0, slot
  const int h = blockIdx.y;
  const long n = (long)a.dv * a.dk;
  const long e = (long)blockIdx.x * 256 + threadIdx.x;
  if (e >= n) return;
  float* st = a.state + ((long)q.w * a.H + h) * n + e;
  float s = q.z == 0 ? 0.f : *st;
  const float* pw = a.pows + (long)h * (LM_TILE + 1);
  float* p = cs + ((long)q.x * a.H + h) * n + e;
  const long step = (long)a.H * n;
  float nxt = *p;
  for (int c = 0; c < q.y; ++c) {
    const float d = nxt;
    if (c + 1 < q.y) nxt = p[step];
    *p = s;
    s = fmaf(s, pw[tiles[q.x + c].y], d);
    p += step;
  }
  *st = s;
}

template <bool F32, int DK, int DV>
__global__ void __launch_bounds__(256)
ret_chunk_out_kernel(RetArgs a, const int4* __restrict__ tiles,
                     const float* __restrict__ cs) {
  using N = Num<F32>;
  using E = typename N::E;
  constexpr int LDK = DK + N::PAD;
  constexpr int LDJ = LM_TILE + N::PAD;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const ColTile<F32, DV> V{(E*)smem};
  E* Pb = V.p + V.SIZE;                     // [PARTS][64][LDJ]
  E* Xb = Pb + Split<F32>::PARTS * LM_TILE * LDJ;   // [PARTS][64][LDK]
  const Split<F32> P{Pb, Pb + LM_TILE * LDJ};
  const Split<F32> X{Xb, Xb + LM_TILE * LDK};       // q, then k, then S

  const int4 t = tiles[blockIdx.y];
  const int h = blockIdx.x;   // heads of a row run together: whole rows stream
  const int tid = threadIdx.x, w = tid >> 6, l = tid & 63;
  const int lr = l & 15, lg = l >> 4;
  const bool aligned = ret_aligned(a);
  const float* pw = a.pows + (long)h * (LM_TILE + 1);
  const E* base = (const E*)a.qkvg + (long)t.x * a.ld;

  auto stage_qk = [&](long off, float mul) {
    stage_rot<F32, DK>(base + off, a, t.z, t.y, aligned,
                       [&](int) { return mul; },
                       [&](int j, int c, float* v) { X.put8(j * LDK + c, v); });
  };
  stage_qk((long)h * a.dk, 1.f);
  ret_values<F32, DV>(V, base + (long)2 * a.H * a.dk + (long)h * a.dv, a, t.y,
                      aligned);
  __syncthreads();
  typename Split<F32>::Frag qf[DK / 32];
  #pragma unroll
  for (int kb = 0; kb < DK / 32; ++kb)
    qf[kb] = X.load((16 * w + lr) * LDK, kb * 32 + lg * 8);
  __syncthreads();
  stage_qk((long)(a.H + h) * a.dk, a.kscale);
  __syncthreads();

  // decayed scores of this wave's 16 rows
  #pragma unroll
  for (int ct = 0; ct < 4; ++ct) {
    f32x4 s = f32x4{0.f, 0.f, 0.f, 0.f};
    if (ct <= w) {
      #pragma unroll
      for (int kb = 0; kb < DK / 32; ++kb)
        s = mma_ss<F32>(qf[kb], X.load((ct * 16 + lr) * LDK, kb * 32 + lg * 8), s);
    }
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * w + 4 * lg + r, j = ct * 16 + lr;
      P.put(i * LDJ + j, j <= i ? s[r] * pw[i - j] : 0.f);
    }
  }

  f32x4 o[DV / 16];                         // against the incoming state
  times_state<F32, DK, DV, LDK>(
      cs + ((long)blockIdx.y * a.H + h) * a.dv * a.dk, a.dv, a.dk, X, o,
      [&](int kb, const typename Split<F32>::Frag& s, f32x4 acc) {
        return mma_ss<F32>(qf[kb], s, acc);
      });
  // gates: all in flight here, used in the epilogue
  E gz[4][DV / 16];
  if (!a.raw) {
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      const E* gate = base + (long)min(16 * w + 4 * lg + r, t.y - 1) * a.ld +
                      (long)2 * a.H * a.dk + (long)(a.H + h) * a.dv;
      #pragma unroll
      for (int i = 0; i < DV / 16; ++i)
        gz[r][i] = gate[min(i * 16 + lr, a.dv - 1)];
    }
  }
  float ss[4] = {0.f, 0.f, 0.f, 0.f};
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    const float d = pw[16 * w + 4 * lg + r + 1];
    #pragma unroll
    for (int i = 0; i < DV / 16; ++i) o[i][r] *= d;
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
  if (a.raw) {
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = 16 * w + 4 * lg + r;
      if (row >= t.y) continue;
      E* dst = (E*)a.out + ((long)(t.x + row) * a.H + h) * a.dv;
      #pragma unroll
      for (int i = 0; i < DV / 16; ++i)
        if (i * 16 + lr < a.dv) dst[i * 16 + lr] = N::down(o[i][r]);
    }
    return;
  }
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    #pragma unroll
    for (int i = 0; i < DV / 16; ++i) ss[r] += o[i][r] * o[i][r];
    ss[r] = 1.0f / sqrtf(sum16(ss[r]) / (float)a.dv + a.eps);
  }
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = 16 * w + 4 * lg + r;
    if (row >= t.y) continue;
    E* dst = (E*)a.out + ((long)(t.x + row) * a.H + h) * a.dv;
    #pragma unroll
    for (int i = 0; i < DV / 16; ++i) {
      const int c = i * 16 + lr;
      if (c < a.dv) {
        const float z = N::up(gz[r][i]);
        dst[c] = N::down(o[i][r] * ss[r] * (z / (1.0f + expf(-z))));
      }
    }
  }
}

// One token of one row and head per block.
template <bool F32, int NT>
__global__ void __launch_bounds__(NT)
ret_decode_kernel(RetArgs a, const int* __restrict__ pos,
                  const int* __restrict__ slot) {
  using N = Num<F32>;
  using E = typename N::E;
  __shared__ float q_s[256], k_s[256], o_s[256], red[NT / 64];
  const int h = blockIdx.x, row = blockIdx.y;
  const int tid = threadIdx.x;
  E* dst = (E*)a.out + ((long)row * a.H + h) * a.dv;
  const int s = slot[row];
  if (s < 0) {
    for (int c = tid; c < a.dv; c += NT) dst[c] = N::down(0.f);
    return;
  }
  const int p = pos[row];
  const E* base = (const E*)a.qkvg + (long)row * a.ld;
  const E* vrow = base + (long)2 * a.H * a.dk + (long)h * a.dv;
  const E* grow = vrow + (long)a.H * a.dv;
  const int half = a.rd >> 1;
  for (int e = tid; e < 2 * a.dk; e += NT) {
    const bool isk = e >= a.dk;
    const int c = isk ? e - a.dk : e;
    const E* head = base + (long)(isk ? a.H + h : h) * a.dk;
    float x = N::up(head[c]);
    if (c < a.rd) {
      const bool low = c < half;
      const int i = low ? c : c - half;
      const float y = N::up(head[low ? c + half : c - half]);
      const float cv = a.cos_t[(long)p * half + i], sv = a.sin_t[(long)p * half + i];
      x = low ? x * cv - y * sv : x * cv + y * sv;
    }
    if (a.silu) x = silu(x);
    (isk ? k_s : q_s)[c] = isk ? x * a.kscale : x;
  }
  __syncthreads();

  auto value = [&](int r) {
    const float v = N::up(vrow[r]);
    return a.silu ? N::up(N::down(silu(v))) : v;
  };
  const float dh = a.dec[2 * h], dl = a.dec[2 * h + 1];
  float* S = a.state + ((long)s * a.H + h) * a.dv * a.dk;
  const bool fresh = p == 0;
  if (a.dk % 4 == 0) {
    int lpr = 1;                            // lanes that share a state row
    while (lpr * 4 < a.dk) lpr <<= 1;
    const int c = (tid & (lpr - 1)) * 4;
    const int rstep = NT / lpr;
    constexpr int RB = 4;
    const bool in = c < a.dk;
    f32x4 kv = f32x4{0.f, 0.f, 0.f, 0.f}, qv = kv;
    if (in) {
      kv = *(const f32x4*)(k_s + c);
      qv = *(const f32x4*)(q_s + c);
    }
    for (int r0 = tid / lpr; r0 < a.dv; r0 += rstep * RB) {
      f32x4 x[RB];
      #pragma unroll
      for (int u = 0; u < RB; ++u) {
        const int r = r0 + u * rstep;
        x[u] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (in && r < a.dv && !fresh) x[u] = *(const f32x4*)(S + (long)r * a.dk + c);
      }
      #pragma unroll
      for (int u = 0; u < RB; ++u) {
        const int r = r0 + u * rstep;
        float d = 0.f;
        if (in && r < a.dv) {
          const float v = value(r);
          #pragma unroll
          for (int j = 0; j < 4; ++j) {
            x[u][j] = fmaf(x[u][j], dh, fmaf(x[u][j], dl, kv[j] * v));
            d = fmaf(x[u][j], qv[j], d);
          }
          *(f32x4*)(S + (long)r * a.dk + c) = x[u];
        }
        for (int o = 1; o < lpr; o <<= 1) d += __shfl_xor(d, o, 64);
        if (c == 0 && r < a.dv) o_s[r] = d;
      }
    }
  } else {
    const int w = tid >> 6, l = tid & 63;
    for (int r = w; r < a.dv; r += NT / 64) {
      const float v = value(r);
      float d = 0.f;
      for (int c = l; c < a.dk; c += 64) {
        float* e = S + (long)r * a.dk + c;
        const float x0 = fresh ? 0.f : *e;
        const float x = fmaf(x0, dh, fmaf(x0, dl, k_s[c] * v));
        *e = x;
        d = fmaf(x, q_s[c], d);
      }
      d = wave_reduce_sum(d);
      if (l == 0) o_s[r] = d;
    }
  }
  __syncthreads();
  if (a.raw) {
    for (int c = tid; c < a.dv; c += NT) dst[c] = N::down(o_s[c]);
    return;
  }
  float qd = 0.f;
  for (int c = tid; c < a.dv; c += NT) qd += o_s[c] * o_s[c];
  qd = wave_reduce_sum(qd);
  if ((tid & 63) == 0) red[tid >> 6] = qd;
  __syncthreads();
  float tot = 0.f;
  #pragma unroll
  for (int i = 0; i < NT / 64; ++i) tot += red[i];
  const float inv = 1.0f / sqrtf(tot / (float)a.dv + a.eps);
  for (int c = tid; c < a.dv; c += NT) {
    const float z = N::up(grow[c]);
    dst[c] = N::down(o_s[c] * inv * (z / (1.0f + expf(-z))));
  }
}

template <bool F32, int DK, int DV>
void launch_prefill(const RetArgs& a, const int4* tiles, int n_tiles,
                    const int4* seqs, int n_seqs, float* cs, hipStream_t st) {
  using N = Num<F32>;
  using S = Split<F32>;
  constexpr size_t es = sizeof(typename N::E);
  constexpr int LDJ = LM_TILE + N::PAD;
  using V = ColTile<F32, DV>;
  constexpr size_t lds1 = es * (V::SIZE + S::PARTS * ColTile<F32, DK>::SIZE);
  constexpr size_t lds2 = es * (V::SIZE + S::PARTS * LM_TILE * LDJ +
                                S::PARTS * LM_TILE * (DK + N::PAD));
  static_assert(lds1 <= 160 * 1024 && lds2 <= 160 * 1024, "exceeds the CU's LDS");
  static const hipError_t attr1 = hipFuncSetAttribute(
      (const void*)ret_chunk_state_kernel<F32, DK, DV>,
      hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds1);
  static const hipError_t attr2 = hipFuncSetAttribute(
      (const void*)ret_chunk_out_kernel<F32, DK, DV>,
      hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds2);
  (void)attr1;
  (void)attr2;
  hipLaunchKernelGGL((ret_chunk_state_kernel<F32, DK, DV>), dim3(a.H, n_tiles),
                     dim3(256), lds1, st, a, tiles, cs);
  hipLaunchKernelGGL(ret_scan_kernel,
                     dim3((unsigned)(((long)a.dv * a.dk + 255) / 256), a.H, n_seqs),
                     dim3(256), 0, st, a, tiles, seqs, cs);
  hipLaunchKernelGGL((ret_chunk_out_kernel<F32, DK, DV>), dim3(a.H, n_tiles),
                     dim3(256), lds2, st, a, tiles, (const float*)cs);
}

template <bool F32, int DK>
void pick_dv(const RetArgs& a, const int4* tiles, int n_tiles, const int4* seqs,
             int n_seqs, float* cs, hipStream_t st) {
  if (a.dv <= 64) launch_prefill<F32, DK, 64>(a, tiles, n_tiles, seqs, n_seqs, cs, st);
  else if (a.dv <= 128) launch_prefill<F32, DK, 128>(a, tiles, n_tiles, seqs, n_seqs, cs, st);
  else launch_prefill<F32, DK, 256>(a, tiles, n_tiles, seqs, n_seqs, cs, st);
}

template <bool F32>
void pick_dk(const RetArgs& a, const int4* tiles, int n_tiles, const int4* seqs,
             int n_seqs, float* cs, hipStream_t st) {
  if (a.dk <= 64) pick_dv<F32, 64>(a, tiles, n_tiles, seqs, n_seqs, cs, st);
  else if (a.dk <= 128) pick_dv<F32, 128>(a, tiles, n_tiles, seqs, n_seqs, cs, st);
  else pick_dv<F32, 256>(a, tiles, n_tiles, seqs, n_seqs, cs, st);
}

template <bool F32>
void run_decode(const RetArgs& a, const int* pos, const int* slot, int R,
                hipStream_t st) {
  // every thread keeps 4 state vectors (16 floats) in flight
  const int need = a.dk * a.dv / 16;
  #define RD_GO(NT)                                                            \
    hipLaunchKernelGGL((ret_decode_kernel<F32, NT>), dim3(a.H, R), dim3(NT), 0, \
                       st, a, pos, slot)
  if (need <= 256) RD_GO(256);
  else if (need <= 512) RD_GO(512);
  else RD_GO(1024);
  #undef RD_GO
}

}  // namespace

void lm_ret_prefill(const RetArgs& a, const int4* tiles, int n_tiles,
                    const int4* seqs, int n_seqs, float* cs, bool f32,
                    hipStream_t stream) {
  if (n_tiles <= 0) return;
  if (f32) pick_dk<true>(a, tiles, n_tiles, seqs, n_seqs, cs, stream);
  else pick_dk<false>(a, tiles, n_tiles, seqs, n_seqs, cs, stream);
}

void lm_ret_decode(const RetArgs& a, const int* pos, const int* slot, int R,
                   bool f32, hipStream_t stream) {
  if (R <= 0) return;
  if (f32) run_decode<true>(a, pos, slot, R, stream);
  else run_decode<false>(a, pos, slot, R, stream);
}
