// Routed feed-forward: sigmoid router with expert groups, or a table of token
// ids, gated experts and a shared expert.
//
// One plan kernel chooses the experts, sorts the (token, place) entries by
// expert and cuts them into tiles; two grouped products follow,
//     act = silu(gate x) * (up x)      rows gathered by token, sorted rows out
//     y   = down act                   sorted rows in, [token][place] out
// and the weighted sum over a token's places is left to the residual norm,
// which reads y once.  Nothing is copied to gather or scatter, the host
// never learns the counts, and the grid has room for the worst case:
// blocks without a tile end at once.
//
// The shared expert is one more expert that takes every token, so a token
// costs the same three launches whatever the design has.

#include "lm.h"
#include "tile.h"
#include "attn.h"

#include <type_traits>

namespace {

// ---- routing --------------------------------------------------------------

// larger float <-> larger unsigned
DEVINL unsigned ordered(float f) {
  const unsigned u = __builtin_bit_cast(unsigned, f);
  return u & 0x80000000u ? ~u : u | 0x80000000u;
}

// One wave chooses one token's experts.  NPL scores a lane; sc: the wave's
// scratch for scores, E floats.  Equal logits: the lower index first.
template <int NPL>
DEVINL void route_token(const MoeArgs& a, int t, float* sc, int l) {
  const float* z = a.z + (long)t * a.ldz;
  float zz[NPL], s[NPL];
  #pragma unroll
  for (int i = 0; i < NPL; ++i) {
    const int e = i * 64 + l;
    zz[i] = e < a.E ? z[e] : 0.f;
    s[i] = sigmoid(zz[i]);
  }
  unsigned long long open = ~0ull;       // groups that may be chosen from
  const int size = a.E / a.groups;
  if (a.keep < a.groups) {
    #pragma unroll
    for (int i = 0; i < NPL; ++i)
      if (i * 64 + l < a.E) sc[i * 64 + l] = s[i];
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    float m1 = 0.f, m2 = 0.f;            // scores are positive
    if (l < a.groups)
      for (int i = 0; i < size; ++i) {
        const float v = sc[l * size + i];
        m2 = fmaxf(m2, fminf(v, m1));
        m1 = fmaxf(m1, v);
      }
    const float mine = m1 + m2;
    int before = 0;
    for (int o = 0; o < a.groups; ++o) {
      const float v = __shfl(mine, o, 64);
      before += v > mine || (v == mine && o < l);
    }
    open = __ballot(l < a.groups && before < a.keep);
  }
  unsigned long long key[NPL];
  #pragma unroll
  for (int i = 0; i < NPL; ++i) {
    const int e = i * 64 + l;
    const bool ok = e < a.E && (open >> min(e / size, 63) & 1);
    key[i] = ok ? (unsigned long long)ordered(zz[i]) << 32 | (0xffffffffu - e) : 0;
  }
  for (int k = 0; k < a.top; ++k) {
    unsigned long long best = 0;
    #pragma unroll
    for (int i = 0; i < NPL; ++i) best = max(best, key[i]);
    #pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const unsigned hi = __shfl_xor((unsigned)(best >> 32), o, 64);
      const unsigned lo = __shfl_xor((unsigned)best, o, 64);
      best = max(best, (unsigned long long)hi << 32 | lo);
    }
    const int e = (int)min(0xffffffffu - (unsigned)best, (unsigned)a.E - 1);
    #pragma unroll
    for (int i = 0; i < NPL; ++i)
      if (i * 64 + l == e) {
        key[i] = 0;
        a.ids[(long)t * a.top + k] = e;
        a.wts[(long)t * a.K + k] = s[i] * a.scale;
      }
  }
  if (a.K > a.top && l == 0)
    a.wts[(long)t * a.K + a.top] = sigmoid(z[a.E]);
}

// Router logits of few tokens (bf16 in, float out): a block has 16 tokens x
// 16 rows of the router, its 16 waves split the depth, so that a row costs
// one memory round trip instead of a walk along it.
__global__ void __launch_bounds__(1024)
moe_logits_kernel(const short* __restrict__ x, const short* __restrict__ r,
                  float* __restrict__ z, int T, int W, int n) {
  using N = Num<false>;
  __shared__ __attribute__((aligned(16))) f32x4 part[16][64];
  const int w = threadIdx.x >> 6, l = threadIdx.x & 63;
  const int lr = l & 15, lg = l >> 4;
  const short* xr = x + (long)min(blockIdx.y * 16 + lr, T - 1) * W;
  const short* rr = r + (long)min(blockIdx.x * 16 + lr, n - 1) * W;
  f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
  constexpr int UN = 4;
  for (int k0 = w * 32 * UN; k0 < W; k0 += 16 * 32 * UN) {
    bf16x8 a[UN], b[UN];
    #pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int c = k0 + 32 * u + 8 * lg;
      a[u] = c < W ? *(const bf16x8*)(rr + c) : bf16x8{};
      b[u] = c < W ? *(const bf16x8*)(xr + c) : bf16x8{};
    }
    #pragma unroll
    for (int u = 0; u < UN; ++u) acc = N::mma(a[u], b[u], acc);
  }
  part[w][l] = acc;
  __syncthreads();
  if (w > 0) return;
  #pragma unroll
  for (int i = 1; i < 16; ++i) acc += part[i][l];
  const int t = blockIdx.y * 16 + lr;
  if (t >= T) return;
  #pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int e = blockIdx.x * 16 + 4 * lg + i;
    if (e < n) z[(long)t * n + e] = acc[i];
  }
}

template <int NPL>
__global__ void __launch_bounds__(256)
moe_route_kernel(MoeArgs a) {
  __shared__ float sc[4][NPL * 64];
  const int w = threadIdx.x >> 6, t = blockIdx.x * 4 + w;
  if (t < a.T) route_token<NPL>(a, t, sc[w], threadIdx.x & 63);
}

// With a table nothing is routed: entry i's expert is read there, and all of
// a token's have equal weights.
DEVINL void look_up(const MoeArgs& a, int i) {
  const long tok = min(max(a.tokens[i / a.top], 0l), a.vocab - 1);
  a.ids[i] = min(max(a.table[tok * a.top + i % a.top], 0), a.E - 1);
  a.wts[i] = 1.0f / (float)a.top;
}

__global__ void __launch_bounds__(256)
moe_table_kernel(MoeArgs a) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < a.T * a.top) look_up(a, i);
}

// One block sorts the entries; ROUTE: and routes the tokens (or looks them up)
// before that.
template <int NPL, bool ROUTE>
__global__ void __launch_bounds__(1024)
moe_plan_kernel(MoeArgs a) {
  __shared__ int cnt[NPL * 64], at[NPL * 64 + 1], tat[NPL * 64 + 1];
  __shared__ float sc[ROUTE ? 16 : 1][NPL * 64];
  const int tid = threadIdx.x, w = tid >> 6, l = tid & 63;
  for (int e = tid; e < NPL * 64; e += 1024) cnt[e] = 0;
  const int n = a.T * a.top;
  if constexpr (ROUTE) {
    if (a.table)
      for (int i = tid; i < n; i += 1024) look_up(a, i);
    else
      for (int t = w; t < a.T; t += 16) route_token<NPL>(a, t, sc[w], l);
  }
  __threadfence_block();
  __syncthreads();
  for (int i = tid; i < n; i += 1024) atomicAdd(&cnt[a.ids[i]], 1);
  __syncthreads();
  if (w == 0) {                        // entries and tiles before each expert
    int c[NPL], cs = 0, ts = 0;
    #pragma unroll
    for (int i = 0; i < NPL; ++i) {
      c[i] = cnt[l * NPL + i];
      cs += c[i];
      ts += (c[i] + a.rows - 1) / a.rows;
    }
    int ci = cs, ti = ts;
    #pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int pc = __shfl_up(ci, o, 64), pt = __shfl_up(ti, o, 64);
      if (l >= o) {
        ci += pc;
        ti += pt;
      }
    }
    int c0 = ci - cs, t0 = ti - ts;
    #pragma unroll
    for (int i = 0; i < NPL; ++i) {
      at[l * NPL + i] = c0;
      tat[l * NPL + i] = t0;
      c0 += c[i];
      t0 += (c[i] + a.rows - 1) / a.rows;
    }
    if (l == 63) {
      at[NPL * 64] = c0;
      tat[NPL * 64] = t0;
    }
  }
  __syncthreads();
  const int routed = tat[NPL * 64];    // tiles of the routed experts
  for (int e = w; e < a.E; e += 16) {
    const int c = cnt[e];
    for (int i = l; i * a.rows < c; i += 64)
      if (tat[e] + i < a.n_tiles)
        a.tiles[tat[e] + i] = int4{e, at[e] + i * a.rows, min(a.rows, c - i * a.rows), 0};
  }
  const int shared = a.K > a.top ? (a.T + a.rows - 1) / a.rows : 0;
  for (int i = tid; routed + i < a.n_tiles; i += 1024)
    a.tiles[routed + i] =
        i < shared ? int4{a.E, n + i * a.rows, min(a.rows, a.T - i * a.rows), 0}
                   : int4{0, 0, 0, 0};
  if (a.K > a.top)
    for (int t = tid; t < a.T; t += 1024) a.order[n + t] = t * a.K + a.top;
  __syncthreads();
  for (int i = tid; i < n; i += 1024) {
    const int e = a.ids[i];
    a.order[atomicAdd(&at[e], 1)] = i / a.top * a.K + i % a.top;
  }
}

// ---- grouped products ------------------------------------------------------

DEVINL float silu(float z) { return z / (1.0f + expf(-z)); }

// What a tile's expert multiplies.  UP: x rows by [gate; up], else act rows
// by down.
template <bool F32, bool UP> struct Expert {
  using E = typename Num<F32>::E;
  const E* w;      // UP: gate rows, the up rows follow n rows further
  int n, k;        // outputs, depth
  DEVINL Expert(const MoeArgs& a, int e) {
    const bool own = e < a.E;
    const int ff = own ? a.ff : a.ffs;
    n = UP ? ff : a.W;
    k = UP ? a.W : ff;
    const void* base = UP ? (own ? a.gu : a.sgu) : (own ? a.down : a.sdown);
    w = (const E*)base + (own ? (long)e * (UP ? 2 : 1) * ff * a.W : 0);
  }
};

// Any size, either precision: 64 entries x 64 outputs a block, 16x16 tiles.
template <bool F32, bool UP>
__global__ void __launch_bounds__(256)
moe_any_kernel(MoeArgs a) {
  using N = Num<F32>;
  using E = typename N::E;
  constexpr int LD = 32 + N::PAD, NB = UP ? 2 : 1;
  __shared__ __attribute__((aligned(16))) E As[64 * LD], Bs[NB][64 * LD];
  __shared__ int ord[64];
  const int4 t = a.tiles[blockIdx.y];
  if (t.z == 0) return;
  const Expert<F32, UP> ex(a, t.x);
  const int n0 = blockIdx.x * 64;
  if (n0 >= ex.n) return;
  const int tid = threadIdx.x, w = tid >> 6, l = tid & 63;
  const int lr = l & 15, lg = l >> 4;
  const bool aligned = ex.k % 8 == 0;
  if (tid < 64) ord[tid] = a.order[t.y + min(tid, t.z - 1)];
  __syncthreads();

  // this thread stages 8 columns of one row of each operand
  const int sr = tid >> 2, sc = (tid & 3) * 8;
  const E* arow = UP ? (const E*)a.x + (long)(ord[sr] / a.K) * a.W
                     : (const E*)a.act + (long)(t.y + min(sr, t.z - 1)) * a.lda;
  const E* brow[NB];
  #pragma unroll
  for (int b = 0; b < NB; ++b)
    brow[b] = ex.w + (long)(b * ex.n + min(n0 + sr, ex.n - 1)) * ex.k;

  f32x4 acc[NB][4];
  #pragma unroll
  for (int b = 0; b < NB; ++b)
    #pragma unroll
    for (int i = 0; i < 4; ++i) acc[b][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  Raw8<F32> ra, rb[NB];
  auto fetch = [&](int k0) {
    ra.load(arow + k0 + sc, ex.k - k0 - sc, aligned);
    #pragma unroll
    for (int b = 0; b < NB; ++b)
      rb[b].load(brow[b] + k0 + sc, ex.k - k0 - sc, aligned);
  };
  fetch(0);
  for (int k0 = 0; k0 < ex.k; k0 += 32) {
    __syncthreads();
    #pragma unroll
    for (int i = 0; i < 8; ++i) {
      As[sr * LD + sc + i] = ra.e[i];
      #pragma unroll
      for (int b = 0; b < NB; ++b) Bs[b][sr * LD + sc + i] = rb[b].e[i];
    }
    __syncthreads();
    if (k0 + 32 < ex.k) fetch(k0 + 32);
    const auto af = N::load(As + (16 * w + lr) * LD, lg * 8);
    #pragma unroll
    for (int b = 0; b < NB; ++b)
      #pragma unroll
      for (int i = 0; i < 4; ++i)
        acc[b][i] = N::mma(af, N::load(Bs[b] + (16 * i + lr) * LD, lg * 8), acc[b][i]);
  }
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = 16 * w + 4 * lg + r;
    if (row >= t.z) continue;
    E* dst = UP ? (E*)a.act + (long)(t.y + row) * a.lda
                : (E*)a.y + (long)ord[row] * a.W;
    #pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = n0 + 16 * i + lr;
      if (c < ex.n)
        dst[c] = N::down(UP ? silu(acc[0][i][r]) * acc[NB - 1][i][r] : acc[0][i][r]);
    }
  }
}

// Few entries per expert (bf16): the time is that of reading the weights.
// A block has 16 outputs of one tile; its 4 waves split the depth, so every
// weight goes from memory to one wave's registers and nowhere else.  The
// entries (up to 64, 16 a column tile) are the product's columns.
template <bool UP>
__global__ void __launch_bounds__(256)
moe_few_kernel(MoeArgs a) {
  using N = Num<false>;
  constexpr int NB = UP ? 2 : 1, NT = 4, UN = 4;
  __shared__ __attribute__((aligned(16))) f32x4 part[3][NB * NT][64];
  const int4 t = a.tiles[blockIdx.y];
  if (t.z == 0) return;
  const Expert<false, UP> ex(a, t.x);
  const int n0 = blockIdx.x * 16;
  if (n0 >= ex.n) return;
  const int w = threadIdx.x >> 6, l = threadIdx.x & 63;
  const int lr = l & 15, lg = l >> 4;
  const int nt = (t.z + 15) / 16;

  const short* wr[NB];
  #pragma unroll
  for (int b = 0; b < NB; ++b)
    wr[b] = ex.w + (long)(b * ex.n + min(n0 + lr, ex.n - 1)) * ex.k;
  const short* xr[NT];
  #pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int e = t.y + min(16 * i + lr, t.z - 1);
    xr[i] = UP ? (const short*)a.x + (long)(a.order[e] / a.K) * a.W
               : (const short*)a.act + (long)e * a.lda;
  }
  f32x4 acc[NB][NT];
  #pragma unroll
  for (int b = 0; b < NB; ++b)
    #pragma unroll
    for (int i = 0; i < NT; ++i) acc[b][i] = f32x4{0.f, 0.f, 0.f, 0.f};

  // wave w takes every fourth span of 32 * UN columns
  for (int k0 = w * 32 * UN; k0 < ex.k; k0 += 4 * 32 * UN) {
    bf16x8 wf[NB][UN];
    #pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int c = k0 + 32 * u + 8 * lg;
      #pragma unroll
      for (int b = 0; b < NB; ++b)
        wf[b][u] = c < ex.k ? *(const bf16x8*)(wr[b] + c) : bf16x8{};
    }
    #pragma unroll
    for (int i = 0; i < NT; ++i) {
      if (i >= nt) continue;
      bf16x8 xf[UN];
      #pragma unroll
      for (int u = 0; u < UN; ++u) {
        const int c = k0 + 32 * u + 8 * lg;
        xf[u] = c < ex.k ? *(const bf16x8*)(xr[i] + c) : bf16x8{};
      }
      #pragma unroll
      for (int u = 0; u < UN; ++u)
        #pragma unroll
        for (int b = 0; b < NB; ++b) acc[b][i] = N::mma(wf[b][u], xf[u], acc[b][i]);
    }
  }
  if (w > 0) {
    #pragma unroll
    for (int b = 0; b < NB; ++b)
      #pragma unroll
      for (int i = 0; i < NT; ++i) part[w - 1][b * NT + i][l] = acc[b][i];
  }
  __syncthreads();
  if (w > 0) return;
  #pragma unroll
  for (int i = 0; i < NT; ++i) {
    if (i >= nt) continue;
    #pragma unroll
    for (int b = 0; b < NB; ++b)
      #pragma unroll
      for (int o = 0; o < 3; ++o) acc[b][i] += part[o][b * NT + i][l];
    const int row = 16 * i + lr;       // entry; outputs n0 + 4 * lg ..
    if (row >= t.z) continue;
    short* dst = UP ? (short*)a.act + (long)(t.y + row) * a.lda
                    : (short*)a.y + (long)a.order[t.y + row] * a.W;
    bf16x4 pk;
    #pragma unroll
    for (int r = 0; r < 4; ++r)
      pk[r] = cvt_bf16(UP ? silu(acc[0][i][r]) * acc[NB - 1][i][r] : acc[0][i][r]);
    // widths are multiples of 8 here
    if (n0 + 4 * lg < ex.n) *(bf16x4*)(dst + n0 + 4 * lg) = pk;
  }
}

// Many entries per expert (bf16, depths that are multiples of 64): 128
// entries x 128 weight rows a block, 4 waves of 64 x 64, 64 columns a step
// copied straight from memory to LDS into the other half of a double buffer.
// Each lane fetches what belongs in its 16 bytes, so the rows' gather and
// the swizzle cost nothing.  UP: the weight rows are 2 x (32 gate, 32 up),
// so a wave's accumulators hold a gate and its up side by side.  The weights
// are the first operand: a lane then has 4 outputs in a row to store.
template <bool UP>
__global__ void __launch_bounds__(256, 2)
moe_many_kernel(MoeArgs a, int gn) {
  using N = Num<false>;
  constexpr int TILE = 128 * 64, COLS = UP ? 64 : 128;
  __shared__ __attribute__((aligned(16))) short lds[2][2 * TILE];
  __shared__ int ord[128];

  // four tiles at a time go to one XCD with all their outputs
  const unsigned xcd = blockIdx.x % 8, idx = blockIdx.x / 8;
  const unsigned in = idx % (4 * gn), group = idx / (4 * gn) * 8 + xcd;
  const int tile = (int)(group * 4 + in % 4), n0 = (int)(in / 4) * COLS;
  if (tile >= a.n_tiles) return;
  const int4 t = a.tiles[tile];
  if (t.z == 0) return;
  const Expert<false, UP> ex(a, t.x);
  if (n0 >= ex.n) return;
  const int tid = threadIdx.x, w = tid >> 6, l = tid & 63;
  const int wm = w >> 1, wn = w & 1;
  if (tid < 128) ord[tid] = a.order[t.y + min(tid, t.z - 1)];
  __syncthreads();

  const short *xs[4], *ws[4];          // the 4 rows this lane copies from
  #pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = (i * 4 + w) * 8 + (l >> 3), c = ((l & 7) ^ (row & 7)) * 8;
    xs[i] = (UP ? (const short*)a.x + (long)(ord[row] / a.K) * a.W
                : (const short*)a.act + (long)(t.y + min(row, t.z - 1)) * a.lda) + c;
    long wrow;
    if constexpr (UP)
      wrow = (long)(row >> 5 & 1) * ex.n + min(n0 + (row >> 6) * 32 + (row & 31), ex.n - 1);
    else
      wrow = min(n0 + row, ex.n - 1);
    ws[i] = ex.w + wrow * ex.k + c;
  }
  auto stage = [&](int buf, int k0) {
    #pragma unroll
    for (int i = 0; i < 4; ++i) {
      glds16(xs[i] + k0, lds[buf] + (i * 4 + w) * 512);
      glds16(ws[i] + k0, lds[buf] + TILE + (i * 4 + w) * 512);
    }
  };
  f32x4 acc[4][4];                     // [weight rows / 16][entries / 16]
  #pragma unroll
  for (int i = 0; i < 4; ++i)
    #pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  stage(0, 0);
  __syncthreads();
  int cur = 0;
  for (int k0 = 0; k0 < ex.k; k0 += 64) {
    if (k0 + 64 < ex.k) stage(cur ^ 1, k0 + 64);
    const short *sx = lds[cur], *sw = lds[cur] + TILE;
    #pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8 xf[4], wf[4];
      const int kb = kk * 4 + (l >> 4);
      #pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int row = 64 * wm + 16 * i + (l & 15);
        xf[i] = *(const bf16x8*)(sx + row * 64 + (kb ^ (row & 7)) * 8);
        const int col = 64 * wn + 16 * i + (l & 15);
        wf[i] = *(const bf16x8*)(sw + col * 64 + (kb ^ (col & 7)) * 8);
      }
      #pragma unroll
      for (int i = 0; i < 4; ++i)
        #pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = N::mma(wf[i], xf[j], acc[i][j]);
    }
    __syncthreads();                   // reads are over, copies have landed
    cur ^= 1;
  }
  #pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int row = 64 * wm + 16 * j + (l & 15);
    if (row >= t.z) continue;
    short* dst = UP ? (short*)a.act + (long)(t.y + row) * a.lda
                    : (short*)a.y + (long)ord[row] * a.W;
    #pragma unroll
    for (int i = 0; i < (UP ? 2 : 4); ++i) {
      const int c = n0 + (UP ? 32 : 64) * wn + 16 * i + 4 * (l >> 4);
      bf16x4 pk;
      #pragma unroll
      for (int r = 0; r < 4; ++r)
        pk[r] = cvt_bf16(UP ? silu(acc[i][j][r]) * acc[(i + 2) % 4][j][r] : acc[i][j][r]);
      if (c < ex.n) *(bf16x4*)(dst + c) = pk;
    }
  }
}

enum Kind { ANY, FEW, MANY };

Kind pick(const MoeArgs& a, bool f32) {
  if (f32 || a.W % 8 || a.ff % 8 || a.ffs % 8) return ANY;
  if ((long)a.T * a.top < 48L * a.E) return FEW;
  return a.W % 64 || a.ff % 64 || a.ffs % 64 ? ANY : MANY;
}

template <int NPL>
void plan(const MoeArgs& a, hipStream_t st) {
  if (a.T <= 32 || (a.table && a.T * a.top <= 1024)) {
    hipLaunchKernelGGL((moe_plan_kernel<NPL, true>), dim3(1), dim3(1024), 0, st, a);
  } else {
    if (a.table)
      hipLaunchKernelGGL(moe_table_kernel, dim3((a.T * a.top + 255) / 256),
                         dim3(256), 0, st, a);
    else
      hipLaunchKernelGGL((moe_route_kernel<NPL>), dim3((a.T + 3) / 4), dim3(256), 0, st, a);
    hipLaunchKernelGGL((moe_plan_kernel<NPL, false>), dim3(1), dim3(1024), 0, st, a);
  }
}

template <bool UP>
void product(const MoeArgs& a, bool f32, hipStream_t st) {
  const int n = UP ? std::max(a.ff, a.ffs) : a.W;
  const Kind kind = pick(a, f32);
  if (kind == MANY) {
    const int gn = (n + (UP ? 63 : 127)) / (UP ? 64 : 128);
    const long groups = (a.n_tiles + 31) / 32 * 8;
    hipLaunchKernelGGL((moe_many_kernel<UP>), dim3((unsigned)(groups * 4 * gn)),
                       dim3(256), 0, st, a, gn);
  } else if (kind == FEW) {
    hipLaunchKernelGGL((moe_few_kernel<UP>), dim3((n + 15) / 16, a.n_tiles),
                       dim3(256), 0, st, a);
  } else {
    const dim3 grid((n + 63) / 64, a.n_tiles);
    if (f32) hipLaunchKernelGGL((moe_any_kernel<true, UP>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((moe_any_kernel<false, UP>), grid, dim3(256), 0, st, a);
  }
}

}  // namespace

void lm_moe_logits(const void* x, const void* r, float* z, int T, int W, int n,
                   hipStream_t st) {
  hipLaunchKernelGGL(moe_logits_kernel, dim3((n + 15) / 16, (T + 15) / 16),
                     dim3(1024), 0, st, (const short*)x, (const short*)r, z, T,
                     W, n);
}

void lm_moe_plan(const MoeArgs& a, hipStream_t st) {
  if (a.T <= 0) return;
  if (a.E <= 64) plan<1>(a, st);
  else if (a.E <= 128) plan<2>(a, st);
  else if (a.E <= 256) plan<4>(a, st);
  else plan<8>(a, st);
}

int lm_moe_rows(const MoeArgs& a, bool f32) {
  return pick(a, f32) == MANY ? 128 : 64;
}

void lm_moe_experts(const MoeArgs& a, bool f32, hipStream_t st) {
  if (a.T <= 0) return;
  product<true>(a, f32, st);
  product<false>(a, f32, st);
}
