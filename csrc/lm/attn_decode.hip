// Decode attention: one new token per row against its paged cache, all
// query heads of a kv head in one block so keys and values are read once.
//
// The block norms q (every split needs it) and, in the split that holds
// the new token, norms k and appends k and v to the cache; the new key is
// scored from registers, so no other block waits for that write.
// LPK lanes share one key (8 elements each), 64/LPK keys go through a wave
// at a time and each lane group keeps its own running softmax; groups,
// waves and splits merge at the end.  The sink joins the last merge.
// The next pass's keys and values are loaded before the current ones are
// used, and the split's page ids wait in LDS, so a pass costs no
// dependent memory round trip.
//
// Window form: a split is a span of the visible keys in order, the kept first
// ones before the window's; a new value is normed over its head; scores pass
// the soft cap and take their distance's bias (from LDS if it fits).
//
// Tied form: one cached row is key and value, so only half the bytes are
// read; every block takes the root mean squares over the whole of q and of
// the new k itself, and the key weights go to the query's side.

#include "lm.h"
#include "tile.h"
#include "attn.h"

namespace {

constexpr float LOG2E = 1.4426950408889634f;
constexpr float NEG = -1e30f;

// 8 elements, normed over the lane group and rounded to the cache's type
template <bool F32, int LPK>
DEVINL void head_norm(float* v, const void* w, int c, int dim, float eps) {
  using N = Num<F32>;
  float q = 0.f;
  #pragma unroll
  for (int i = 0; i < 8; ++i) q += v[i] * v[i];
  q = group_sum<LPK>(q);
  if (!w) return;
  const float inv = 1.0f / sqrtf(q / (float)dim + eps);
  #pragma unroll
  for (int i = 0; i < 8; ++i)
    if (c + i < dim)
      v[i] = N::up(N::down(v[i] * inv * N::up(((const typename N::E*)w)[c + i])));
}

// over its root mean square, without weights
template <bool F32, int LPK>
DEVINL void unit_norm(float* v, int dim, float eps) {
  float q = 0.f;
  #pragma unroll
  for (int i = 0; i < 8; ++i) q += v[i] * v[i];
  const float inv = 1.0f / sqrtf(group_sum<LPK>(q) / (float)dim + eps);
  #pragma unroll
  for (int i = 0; i < 8; ++i) v[i] *= inv;
}

// What norms the new token's q (its temperature included) and k: a block of
// 256 threads reads both rows.
template <bool F32>
DEVINL void tied_factors(const AttnArgs& a, const typename Num<F32>::E* qkv,
                         int p, bool aligned, float (&red)[2][4], float& inv_q,
                         float& inv_k) {
  const int tid = threadIdx.x, w = tid >> 6;
  const int nq = a.H * a.dim, nk = a.G * a.dim;
  float sq = 0.f, sk = 0.f;
  for (int e = tid * 8; e < nq + nk; e += 256 * 8) {
    float v[8], z = 0.f;              // the span of q ends at a multiple of 8
    if (aligned) {                    // if heads do; k follows q
      load8<F32>(qkv + e, 8, true, v);
      #pragma unroll
      for (int i = 0; i < 8; ++i) z += v[i] * v[i];
      if (e < nq) sq += z;
      else sk += z;
    } else {
      #pragma unroll
      for (int i = 0; i < 8; ++i)
        if (e + i < nq + nk) {
          const float u = Num<F32>::up(qkv[e + i]);
          if (e + i < nq) sq += u * u;
          else sk += u * u;
        }
    }
  }
  sq = group_sum<64>(sq);
  sk = group_sum<64>(sk);
  if ((tid & 63) == 0) {
    red[0][w] = sq;
    red[1][w] = sk;
  }
  __syncthreads();
  sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
  sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  inv_q = temperature(a, p) / sqrtf(sq / (float)nq + a.eps);
  inv_k = 1.0f / sqrtf(sk / (float)nk + a.eps);
}

enum Form { PLAIN, TIED_KV, WINDOW };

template <bool F32, int LPK, int HGC, int FORM>
__global__ void __launch_bounds__(256)
attn_decode_kernel(AttnArgs a, const int* __restrict__ pos,
                   const int* __restrict__ slot, int nsplit,
                   float* __restrict__ ws) {
  using N = Num<F32>;
  using E = typename N::E;
  constexpr int KPW = 64 / LPK;      // keys per wave and pass
  constexpr int KB = F32 ? 2 : 4;    // keys per lane group and pass
  constexpr int TABS = 512;          // page ids kept in LDS
  constexpr int BIAS = 512;          // and entries of a head's bias
  constexpr bool TIED = FORM == TIED_KV, WIN = FORM == WINDOW;
  __shared__ int tab_s[TABS];
  __shared__ float bias_s[WIN ? HGC : 1][WIN ? BIAS : 1];
  constexpr int NP = 4 * KPW;        // partial results of a block
  __shared__ __attribute__((aligned(16))) float acc_s[HGC][NP][LPK * 8];
  __shared__ float m_s[HGC][NP], l_s[HGC][NP];

  const int split = blockIdx.x, row = blockIdx.z;
  const int hg = a.H / a.G, nhc = (hg + HGC - 1) / HGC;
  const int g = blockIdx.y / nhc, hc = blockIdx.y % nhc;
  const int nh = min(HGC, hg - hc * HGC);     // heads of this block
  const int h0 = g * hg + hc * HGC;
  const int tid = threadIdx.x, w = tid >> 6, l = tid & 63;
  const int grp = l / LPK, c = (l % LPK) * 8;
  const bool aligned = a.dim % 8 == 0 && a.vdim % 8 == 0;
  E* out = (E*)a.out + (long)row * a.ldo;

  const int s = slot[row];
  if (s < 0) {                        // idle row: a defined, unused output
    if (split == 0)
      for (int i = tid; i < nh * a.vdim; i += 256)
        out[(long)h0 * a.vdim + i] = N::down(0.f);
    if (nsplit > 1)
      for (int i = tid; i < nh * (a.vdim + 2); i += 256)
        ws[(((long)row * a.H + h0 + i / (a.vdim + 2)) * nsplit + split) *
               (a.vdim + 2) + i % (a.vdim + 2)] = 0.f;
    return;
  }
  const int p = pos[row];
  // visible keys in order: `nk` kept ones from 0 on, then those from cs on;
  // u counts them from cs - nk, so that u is the position of the latter
  const int cs = first_seen(a, p), nk = WIN ? min(a.keep, cs) : 0;
  const int u0 = cs - nk;
  const int nkeys = p - u0 + 1;
  const int per = (nkeys + nsplit - 1) / nsplit;
  const int jb = u0 + split * per;
  const int je = min(jb + per, p + 1);        // may be <= jb: empty split
  const bool has_new = jb <= p && je == p + 1;
  auto place = [&](int u) { return WIN && u < cs ? u - u0 : u; };
  const int* tab = a.table + (long)s * a.max_pages;
  const E* qkv = (const E*)a.qkv + (long)row * a.ld;

  float q[HGC][8], acc[HGC][8], m[HGC], ls[HGC], slope2[HGC];
  const float scale2 = a.scale * LOG2E;
  float inv_q = 1.f, inv_k = 1.f;     // tied form: of the whole rows
  if constexpr (TIED) {
    __shared__ float red[2][4];
    tied_factors<F32>(a, qkv, p, aligned, red, inv_q, inv_k);
  }
  #pragma unroll
  for (int i = 0; i < HGC; ++i) {
    const int h = h0 + min(i, nh - 1);
    load8<F32>(qkv + (long)h * a.dim + c, a.dim - c, aligned, q[i]);
    if constexpr (TIED) {
      float wq[8], wk[8];
      load8<F32>((const E*)a.qw + (long)h * a.dim + c, a.dim - c, aligned, wq);
      load8<F32>((const E*)a.kw + (long)g * a.dim + c, a.dim - c, aligned, wk);
      #pragma unroll
      for (int j = 0; j < 8; ++j)
        q[i][j] = N::up(N::down(q[i][j] * (inv_q * wq[j] * wk[j])));
    } else {
      head_norm<F32, LPK>(q[i], a.qw, c, a.dim, a.eps);
    }
    slope2[i] = a.slopes ? a.slopes[h] * LOG2E : 0.f;
    m[i] = NEG;
    ls[i] = 0.f;
    #pragma unroll
    for (int j = 0; j < 8; ++j) acc[i][j] = 0.f;
  }

  const bool bias_lds = a.n_bias <= BIAS;
  const float* bias_g[HGC];
  if constexpr (WIN) {
    #pragma unroll
    for (int i = 0; i < HGC; ++i)
      bias_g[i] = a.bias + (long)(h0 + min(i, nh - 1)) * a.n_bias;
    if (bias_lds) {
      #pragma unroll
      for (int i = 0; i < HGC; ++i)
        for (int d = tid; d < a.n_bias; d += 256) bias_s[i][d] = bias_g[i][d];
    }
  }
  const SoftCap cap(a, LOG2E);
  // scores of head i in base 2, at distances dj
  auto windowed = [&](int i, float (&x)[KB], const float (&dj)[KB]) {
    float b[KB], most = 0.f;
    #pragma unroll
    for (int u = 0; u < KB; ++u) {
      const int d = min((int)dj[u], a.n_bias - 1);
      b[u] = (bias_lds ? bias_s[i][d] : bias_g[i][d]) * LOG2E;
      most = fmaxf(most, fabsf(x[u]));
    }
    if constexpr (F32) {
      #pragma unroll
      for (int u = 0; u < KB; ++u) {
        float y = x[u] * a.scale;
        if (a.softcap > 0.f) y = a.softcap * tanhf(y / a.softcap);
        x[u] = fmaf(y, LOG2E, b[u]);
      }
    } else if (cap.small(most)) {
      #pragma unroll
      for (int u = 0; u < KB; ++u) x[u] = cap.near(x[u], b[u]);
    } else {
      #pragma unroll
      for (int u = 0; u < KB; ++u) x[u] = cap.any(x[u], b[u]);
    }
  };

  // kf: scale of a key's scores, dj: its distance
  auto fold = [&](const auto& k, const auto& v, const bool (&ok)[KB],
                  const float (&kf)[KB], const float (&dj)[KB]) {
    #pragma unroll
    for (int i = 0; i < HGC; ++i) {
      float sc[KB], mx = m[i];
      #pragma unroll
      for (int u = 0; u < KB; ++u) {
        float d = 0.f;
        #pragma unroll
        for (int j = 0; j < 8; ++j) d = fmaf(q[i][j], k[u][j], d);
        sc[u] = group_sum<LPK>(d);
      }
      if constexpr (WIN) windowed(i, sc, dj);
      #pragma unroll
      for (int u = 0; u < KB; ++u) {
        if constexpr (!WIN) sc[u] = sc[u] * kf[u] - slope2[i] * dj[u];
        sc[u] = ok[u] ? sc[u] : NEG;
        mx = fmaxf(mx, sc[u]);
      }
      const float al = exp2f(m[i] - mx);
      m[i] = mx;
      float e[KB], es = 0.f;
      #pragma unroll
      for (int u = 0; u < KB; ++u) {
        e[u] = ok[u] ? exp2f(sc[u] - mx) : 0.f;
        es += e[u];
      }
      ls[i] = ls[i] * al + es;
      #pragma unroll
      for (int j = 0; j < 8; ++j) {
        float t = acc[i][j] * al;
        #pragma unroll
        for (int u = 0; u < KB; ++u) t = fmaf(e[u], v[u][j], t);
        acc[i][j] = t;
      }
    }
  };

  const int jc = min(je, p + 1);              // p itself is not cached yet
  const int pg0 = max(jb, cs) / LM_PAGE;      // pages of kept keys aside
  const int npg = jc > max(jb, cs) ? (jc - 1) / LM_PAGE - pg0 + 1 : 0;
  const bool in_lds = npg <= TABS;
  if (in_lds || WIN) {
    for (int i = tid; in_lds && i < npg; i += 256) tab_s[i] = tab[pg0 + i];
    __syncthreads();
  }
  // the new token's key and value, in every lane group of the split that
  // has it; the group whose turn it is takes them from here
  Raw8<F32> knew, vnew;
  if (has_new) {
    float k0[8];
    load8<F32>(qkv + (long)(a.H + g) * a.dim + c, a.dim - c, aligned, k0);
    if constexpr (!TIED) {
      vnew.load(qkv + (long)(a.H + a.G) * a.dim + (long)g * a.vdim + c,
                a.vdim - c, aligned);
      head_norm<F32, LPK>(k0, a.kw, c, a.dim, a.eps);
      if constexpr (WIN) {
        if (a.v_norm) {
          float v0[8];
          #pragma unroll
          for (int j = 0; j < 8; ++j) v0[j] = vnew[j];
          unit_norm<F32, LPK>(v0, a.vdim, a.eps);
          #pragma unroll
          for (int j = 0; j < 8; ++j) vnew.e[j] = N::down(v0[j]);
        }
      }
    }
    #pragma unroll
    for (int j = 0; j < 8; ++j) knew.e[j] = N::down(k0[j]);
    if (w == 0 && grp == 0 && hc == 0) {
      const long page = tab[p / LM_PAGE];
      const long cell = (page * a.G + g) * LM_PAGE + p % LM_PAGE;
      store8<F32>((E*)a.kc + cell * a.dim + c, a.dim - c, aligned, k0);
      if constexpr (TIED) {
        if (g == 0 && c == 0) a.ks[page * LM_PAGE + p % LM_PAGE] = inv_k;
      } else {
        float v0[8];
        #pragma unroll
        for (int j = 0; j < 8; ++j) v0[j] = vnew[j];
        store8<F32>((E*)a.vc + cell * a.vdim + c, a.vdim - c, aligned, v0);
      }
    }
  }
  Raw8<F32> kn[KB], vn[TIED ? 1 : KB];
  bool okn[KB];
  float kfn[KB], djn[KB];
  auto fetch = [&](int j0) {
    #pragma unroll
    for (int u = 0; u < KB; ++u) {
      const int v = j0 + (u * 4 + w) * KPW + grp, j = place(v);
      okn[u] = v < jc;
      const bool cached = v < min(jc, p);
      long cell = 0, tok = 0;
      if (cached) {
        const int page = in_lds && v >= cs ? tab_s[j / LM_PAGE - pg0]
                                           : tab[j / LM_PAGE];
        cell = ((long)page * a.G + g) * LM_PAGE + j % LM_PAGE;
        tok = (long)page * LM_PAGE + j % LM_PAGE;
      }
      kn[u].load((const E*)a.kc + cell * a.dim + c, cached ? a.dim - c : 0, aligned);
      kfn[u] = scale2;
      djn[u] = (float)(p - j);
      if constexpr (TIED) {
        const float f = a.ks[tok];    // token 0's where none is cached
        kfn[u] *= cached ? f : inv_k;
      } else {
        vn[u].load((const E*)a.vc + cell * a.vdim + c, cached ? a.vdim - c : 0, aligned);
      }
      if (v == p && okn[u]) {
        kn[u] = knew;
        if constexpr (!TIED) vn[u] = vnew;
      }
    }
  };
  constexpr int STEP = 4 * KPW * KB;
  if (jb < jc) fetch(jb);
  for (int j0 = jb; j0 < jc; j0 += STEP) {
    Raw8<F32> k[KB], v[TIED ? 1 : KB];
    bool ok[KB];
    float kf[KB], dj[KB];
    #pragma unroll
    for (int u = 0; u < KB; ++u) {
      k[u] = kn[u];
      if constexpr (!TIED) v[u] = vn[u];
      ok[u] = okn[u];
      kf[u] = kfn[u];
      dj[u] = djn[u];
    }
    if (j0 + STEP < jc) fetch(j0 + STEP);
    if constexpr (TIED) fold(k, k, ok, kf, dj);
    else fold(k, v, ok, kf, dj);
  }
  // every lane group's partial meets in LDS
  #pragma unroll
  for (int i = 0; i < HGC; ++i) {
    float* d = acc_s[i][w * KPW + grp] + c;
    *(f32x4*)d = *(const f32x4*)acc[i];
    *(f32x4*)(d + 4) = *(const f32x4*)(acc[i] + 4);
    if (c == 0) {
      m_s[i][w * KPW + grp] = m[i];
      l_s[i][w * KPW + grp] = ls[i];
    }
  }
  __syncthreads();
  for (int t = tid; t < nh * a.vdim; t += 256) {
    const int i = t / a.vdim, d = t % a.vdim;
    float mn = NEG;
    #pragma unroll
    for (int x = 0; x < NP; ++x) mn = fmaxf(mn, m_s[i][x]);
    float lt = 0.f, av = 0.f;
    #pragma unroll
    for (int x = 0; x < NP; ++x) {
      const float f = exp2f(m_s[i][x] - mn);
      lt += l_s[i][x] * f;
      av += acc_s[i][x][d] * f;
    }
    if (nsplit == 1) {
      if (a.has_sink) {
        const float sk = sink_score<F32>(a, h0 + i) * LOG2E;
        const float mt = fmaxf(mn, sk);
        const float f = exp2f(mn - mt);
        lt = lt * f + exp2f(sk - mt);
        av *= f;
      }
      if (a.gate)
        av *= sigmoid(N::up(((const E*)a.gate)[(long)row * a.ld +
                                               (long)(h0 + i) * a.vdim + d]));
      out[(long)(h0 + i) * a.vdim + d] = N::down(av / lt * a.out_scale);
    } else {
      float* o = ws + (((long)row * a.H + h0 + i) * nsplit + split) * (a.vdim + 2);
      o[2 + d] = av;
      if (d == 0) {
        o[0] = mn;
        o[1] = lt;
      }
    }
  }
}

// Tied form in bf16, head sizes that are multiples of 8 up to 128: both
// products on the matrix cores, up to 16 heads of a kv head a block.
//
// A wave takes every fourth page of its split, on its own: the page goes from
// memory to registers in the layout of the first product's operand, K Q^T
// (a lane then has 16 keys' scores of one head), and from there to the
// wave's LDS image, where transpose reads make the second one's, V^T P.  The
// order of keys within that product is the order in which the scores lie,
// so the weights (hi + lo bf16) are operands as they are.  The next page is
// loaded as soon as the scores are done.
template <int DK>
__global__ void __launch_bounds__(256, 2)
attn_decode_tied_kernel(AttnArgs a, const int* __restrict__ pos,
                        const int* __restrict__ slot, int nsplit,
                        float* __restrict__ ws) {
  using N = Num<false>;
  constexpr int KS = DK / 32, DT = DK / 16;      // depth steps, value tiles
  constexpr int LDO = DK + 4;
  __shared__ __attribute__((aligned(16))) short img[4][64 * DK];
  __shared__ float red[2][4], m_s[4][16], l_s[4][16];
  static_assert(sizeof(float) * 4 * 16 * LDO <= sizeof(img), "merge");

  const int split = blockIdx.x, row = blockIdx.z;
  const int hg = a.H / a.G, nhc = (hg + 15) / 16;
  const int g = blockIdx.y / nhc, hc = blockIdx.y % nhc;
  const int nh = min(16, hg - hc * 16), h0 = g * hg + hc * 16;
  const int tid = threadIdx.x, w = tid >> 6, l = tid & 63;
  const int lr = l & 15, lg = l >> 4;
  short* out = (short*)a.out + (long)row * a.ldo;

  const int s = slot[row];
  if (s < 0) {                        // idle row: a defined, unused output
    if (split == 0)
      for (int i = tid; i < nh * a.dim; i += 256) out[(long)h0 * a.dim + i] = 0;
    if (nsplit > 1)
      for (int i = tid; i < nh * (a.dim + 2); i += 256)
        ws[(((long)row * a.H + h0 + i / (a.dim + 2)) * nsplit + split) *
               (a.dim + 2) + i % (a.dim + 2)] = 0.f;
    return;
  }
  const int p = pos[row];
  const int cs = a.size ? p - p % a.size : 0;
  const int pg_lo = cs / LM_PAGE, npg = p / LM_PAGE - pg_lo + 1;
  const int per = (npg + nsplit - 1) / nsplit;
  const int pb = pg_lo + split * per, pe = min(pb + per, pg_lo + npg);
  const int* tab = a.table + (long)s * a.max_pages;
  const short* qkv = (const short*)a.qkv + (long)row * a.ld;
  const short* knew = qkv + (long)(a.H + g) * a.dim;

  // the ids of this wave's first 64 pages, one a lane
  const int mine = pb + w + 4 * l;
  const int pid = mine < pe ? tab[mine] : 0;
  auto page_of = [&](int it) {
    const int x = __shfl(pid, it & 63, 64);
    return it < 64 ? x : tab[pb + w + 4 * it];
  };
  bf16x8 kr[4][KS];
  f32x4 kf[4];
  auto fetch = [&](int pg, long page) {
    const short* base = (const short*)a.kc + (page * a.G + g) * LM_PAGE * a.dim;
    #pragma unroll
    for (int t = 0; t < 4; ++t) {
      const int j = 16 * t + lr;
      // the new token is not read from the cache, nor what lies behind it
      const short* src = pg * LM_PAGE + j < p ? base + (long)j * a.dim : knew;
      #pragma unroll
      for (int k = 0; k < KS; ++k)
        kr[t][k] = *(const bf16x8*)(src + min(32 * k + 8 * lg, a.dim - 8));
      kf[t] = *(const f32x4*)(a.ks + page * LM_PAGE + 16 * t + 4 * lg);
    }
  };
  int it = 0, pg = pb + w;
  if (pg < pe) fetch(pg, page_of(0));

  float inv_q, inv_k;
  tied_factors<false>(a, qkv, p, true, red, inv_q, inv_k);
  bf16x8 qf[KS];
  const int h = h0 + min(lr, nh - 1);
  #pragma unroll
  for (int k = 0; k < KS; ++k) {
    const int c = 32 * k + 8 * lg;
    float q[8], wq[8], wk[8];
    load8<false>(qkv + (long)h * a.dim + c, a.dim - c, true, q);
    load8<false>((const short*)a.qw + (long)h * a.dim + c, a.dim - c, true, wq);
    load8<false>((const short*)a.kw + (long)g * a.dim + c, a.dim - c, true, wk);
    #pragma unroll
    for (int i = 0; i < 8; ++i) qf[k][i] = cvt_bf16(q[i] * (inv_q * wq[i] * wk[i]));
  }
  const float scale2 = a.scale * LOG2E;
  const float slope2 = a.slopes ? a.slopes[h] * LOG2E : 0.f;

  // the append, by the block whose split ends with the new token
  if (pe == pg_lo + npg && pb < pe && hc == 0) {
    const long page = tab[p / LM_PAGE];
    const int j = p % LM_PAGE;
    short* dst = (short*)a.kc + ((page * a.G + g) * LM_PAGE + j) * a.dim;
    if (tid * 8 < a.dim) *(bf16x8*)(dst + tid * 8) = *(const bf16x8*)(knew + tid * 8);
    if (g == 0 && tid == 0) a.ks[page * LM_PAGE + j] = inv_k;
  }

  float m = NEG, ls = 0.f;
  f32x4 o[DT];
  #pragma unroll
  for (int i = 0; i < DT; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  short* im = img[w];
  // transpose reads: this lane's 8 bytes of rows 4 lg .. 4 lg + 3
  const int tr_j = 4 * lg + (lr >> 2);
  const unsigned tr0 = lds_byte_off(im) + tr_j * (DK * 2) + (l & 1) * 8;
  const unsigned trc = tied_chunk<DK>(tr_j, (l & 3) >> 1) * 16;

  for (; pg < pe; pg += 4, ++it) {
    const int j0 = pg * LM_PAGE;
    const bool last = j0 + LM_PAGE > p;
    #pragma unroll
    for (int t = 0; t < 4; ++t)
      #pragma unroll
      for (int k = 0; k < KS; ++k) {
        if (last && j0 + 16 * t + lr > p) kr[t][k] = bf16x8{};
        if (DK > a.dim && 32 * k + 8 * lg >= a.dim) kr[t][k] = bf16x8{};
        *(bf16x8*)(im + (16 * t + lr) * DK +
                   tied_chunk<DK>(16 * t + lr, 4 * k + lg) * 8) = kr[t][k];
      }
    f32x4 sc[4];
    #pragma unroll
    for (int t = 0; t < 4; ++t) {
      sc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
      #pragma unroll
      for (int k = 0; k < KS; ++k) sc[t] = N::mma(kr[t][k], qf[k], sc[t]);
    }
    const bool edge = last || j0 < cs;
    const float d0 = slope2 * (float)(j0 + 4 * lg - p);
    float mx = NEG;
    #pragma unroll
    for (int t = 0; t < 4; ++t)
      #pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = j0 + 16 * t + 4 * lg + r;
        const float f = last && j == p ? inv_k : kf[t][r];
        float x = sc[t][r] * (f * scale2) + fmaf(slope2, (float)(16 * t + r), d0);
        if (edge) x = j <= p && j >= cs ? x : NEG;
        sc[t][r] = x;
        mx = fmaxf(mx, x);
      }
    if (pg + 4 < pe) fetch(pg + 4, page_of(it + 1));
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    // every page of a split has a key that the token sees
    const float mn = fmaxf(m, mx), al = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    ls *= al;
    bf16x8 hi[2], lo[2];
    #pragma unroll
    for (int t = 0; t < 4; ++t)
      #pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float e = __builtin_amdgcn_exp2f(sc[t][r] - mn);
        const short eh = cvt_bf16(e);
        ls += e;
        hi[t >> 1][4 * (t & 1) + r] = eh;
        lo[t >> 1][4 * (t & 1) + r] = cvt_bf16(e - bf2f(eh));
      }
    #pragma unroll
    for (int i = 0; i < DT; ++i) o[i] *= al;
    // the wave reads what its own lanes wrote; LDS keeps their order
    asm volatile("" ::: "memory");
    __builtin_amdgcn_wave_barrier();
    #pragma unroll
    for (int i = 0; i < DT; i += 2) {
      auto at = [&](int ii, int b, int u) {
        return tr0 + (unsigned)(32 * b + 16 * u) * (DK * 2) +
               (trc ^ (unsigned)(2 * ii * 16));
      };
      const bf16x8_quad v = tr_read_quad(
          at(i, 0, 0), at(i, 0, 1), at(i, 1, 0), at(i, 1, 1), at(i + 1, 0, 0),
          at(i + 1, 0, 1), at(i + 1, 1, 0), at(i + 1, 1, 1));
      #pragma unroll
      for (int b = 0; b < 2; ++b) {
        o[i] = N::mma(v.f[b], hi[b], o[i]);
        o[i + 1] = N::mma(v.f[2 + b], hi[b], o[i + 1]);
        o[i] = N::mma(v.f[b], lo[b], o[i]);
        o[i + 1] = N::mma(v.f[2 + b], lo[b], o[i + 1]);
      }
    }
    asm volatile("" ::: "memory");
    __builtin_amdgcn_wave_barrier();
  }

  // the waves' partial results meet in LDS
  ls += __shfl_xor(ls, 16, 64);
  ls += __shfl_xor(ls, 32, 64);
  __syncthreads();
  float* os = (float*)img[0] + w * 16 * LDO;
  #pragma unroll
  for (int i = 0; i < DT; ++i) *(f32x4*)(os + lr * LDO + 16 * i + 4 * lg) = o[i];
  if (lg == 0) {
    m_s[w][lr] = m;
    l_s[w][lr] = ls;
  }
  __syncthreads();
  for (int t = tid; t < nh * a.dim; t += 256) {
    const int i = t / a.dim, d = t % a.dim;
    float mn = NEG, lt = 0.f, av = 0.f;
    #pragma unroll
    for (int x = 0; x < 4; ++x) mn = fmaxf(mn, m_s[x][i]);
    #pragma unroll
    for (int x = 0; x < 4; ++x) {
      const float f = exp2f(m_s[x][i] - mn);
      lt += l_s[x][i] * f;
      av += ((const float*)img[0])[(x * 16 + i) * LDO + d] * f;
    }
    if (nsplit == 1) {
      if (a.has_sink) {
        const float sk = sink_score<false>(a, h0 + i) * LOG2E;
        const float mt = fmaxf(mn, sk), f = exp2f(mn - mt);
        lt = lt * f + exp2f(sk - mt);
        av *= f;
      }
      if (a.gate)
        av *= sigmoid(bf2f(((const short*)a.gate)[(long)row * a.ld +
                                                  (long)(h0 + i) * a.dim + d]));
      out[(long)(h0 + i) * a.dim + d] = cvt_bf16(av / lt * a.out_scale);
    } else {
      float* q = ws + (((long)row * a.H + h0 + i) * nsplit + split) * (a.dim + 2);
      q[2 + d] = av;
      if (d == 0) {
        q[0] = mn;
        q[1] = lt;
      }
    }
  }
}

// One block per (row, head); lane i weighs split i (at most 64).  Groups of
// nd threads (vdim rounded up to whole waves) share the splits.
template <bool F32>
__global__ void __launch_bounds__(512)
attn_combine_kernel(AttnArgs a, const int* __restrict__ slot, int nsplit,
                    const float* __restrict__ ws) {
  using N = Num<F32>;
  using E = typename N::E;
  const int h = blockIdx.x, row = blockIdx.y;
  const int l = threadIdx.x & 63;
  const int st = a.vdim + 2;
  const float* p = ws + ((long)row * a.H + h) * nsplit * st;
  const bool on = l < nsplit;
  const float mi = on ? p[l * st] : NEG, li = on ? p[l * st + 1] : 0.f;
  const float sk = a.has_sink ? sink_score<F32>(a, h) * LOG2E : NEG;
  const bool idle = slot[row] < 0;            // its output is already set
  const float mn = wave_reduce_max(fmaxf(mi, sk));
  const float f = on ? exp2f(mi - mn) : 0.f;
  const float lt = group_sum<64>(li * f) + (a.has_sink ? exp2f(sk - mn) : 0.f);
  const float inv = 1.0f / lt;
  __shared__ float part_s[512];
  const int nd = (a.vdim + 63) / 64 * 64, parts = 512 / nd;
  const int part = threadIdx.x / nd, d = threadIdx.x % nd;
  const int dc = min(d, a.vdim - 1);
  const bool mine = part == 0 && d < a.vdim && !idle;
  float gate = 1.f;                           // on its way meanwhile
  if (a.gate && mine)
    gate = sigmoid(N::up(((const E*)a.gate)[(long)row * a.ld +
                                            (long)h * a.vdim + d]));
  float av = 0.f;
  if (part < parts) {
    #pragma unroll 8
    for (int i = part; i < nsplit; i += parts)
      av = fmaf(p[i * st + 2 + dc], __shfl(f, i, 64), av);
  }
  part_s[threadIdx.x] = av;
  __syncthreads();
  if (!mine) return;
  for (int i = 1; i < parts; ++i) av += part_s[i * nd + d];
  ((E*)a.out)[(long)row * a.ldo + (long)h * a.vdim + d] =
      N::down(av * inv * gate * a.out_scale);
}

template <bool F32, int LPK, int FORM>
void pick_heads(const AttnArgs& a, const int* pos, const int* slot, int R,
                int nsplit, float* ws, hipStream_t st) {
  const int hg = a.H / a.G;
  #define AD_GO(HGC)                                                           \
    hipLaunchKernelGGL((attn_decode_kernel<F32, LPK, HGC, FORM>),              \
                       dim3(nsplit, a.G * ((hg + HGC - 1) / HGC), R),          \
                       dim3(256), 0, st, a, pos, slot, nsplit, ws)
  if (hg == 1) AD_GO(1);
  else if (hg == 2) AD_GO(2);
  else AD_GO(4);
  #undef AD_GO
}

template <bool F32, int LPK>
void pick_form(const AttnArgs& a, const int* pos, const int* slot, int R,
               int nsplit, float* ws, hipStream_t st) {
  if (a.ks) pick_heads<F32, LPK, TIED_KV>(a, pos, slot, R, nsplit, ws, st);
  else if (a.bias) pick_heads<F32, LPK, WINDOW>(a, pos, slot, R, nsplit, ws, st);
  else pick_heads<F32, LPK, PLAIN>(a, pos, slot, R, nsplit, ws, st);
}

template <bool F32>
void run_decode(const AttnArgs& a, const int* pos, const int* slot, int R,
                int nsplit, float* ws, hipStream_t st) {
  const int d = std::max(a.dim, a.vdim);
  if (!F32 && lm_attn_decode_tied_mfma(a)) {
    const dim3 grid(nsplit, a.G * ((a.H / a.G + 15) / 16), R);
    if (d <= 64)
      hipLaunchKernelGGL((attn_decode_tied_kernel<64>), grid, dim3(256), 0, st,
                         a, pos, slot, nsplit, ws);
    else
      hipLaunchKernelGGL((attn_decode_tied_kernel<128>), grid, dim3(256), 0, st,
                         a, pos, slot, nsplit, ws);
  }
  else if (d <= 32) pick_form<F32, 4>(a, pos, slot, R, nsplit, ws, st);
  else if (d <= 64) pick_form<F32, 8>(a, pos, slot, R, nsplit, ws, st);
  else if (d <= 128) pick_form<F32, 16>(a, pos, slot, R, nsplit, ws, st);
  else pick_form<F32, 32>(a, pos, slot, R, nsplit, ws, st);
  if (nsplit > 1)
    hipLaunchKernelGGL((attn_combine_kernel<F32>), dim3(a.H, R),
                       dim3(512), 0, st, a, slot, nsplit, ws);
}

}  // namespace

bool lm_attn_decode_tied_mfma(const AttnArgs& a) {
  return a.ks && a.dim % 8 == 0 && a.dim <= 128;
}

void lm_attn_decode(const AttnArgs& a, const int* pos, const int* slot, int R,
                    int nsplit, float* ws, bool f32, hipStream_t stream) {
  if (R <= 0) return;
  if (f32) run_decode<true>(a, pos, slot, R, nsplit, ws, stream);
  else run_decode<false>(a, pos, slot, R, nsplit, ws, stream);
}
