// The bf16 prompt-attention kernel for head sizes that are multiples of 8
// up to 128 (attn.hip serves every other size and float32).
//
// A block owns one tile of up to 64 prompt rows for HPB query heads of one
// kv head; each head's rows are two waves of 32.  All 2*HPB waves share the
// staged page, so grouped heads pay for keys and values once.
//
//  * S^T = K Q^T with 32x32x16 MFMAs: a lane holds one query's scores for
//    32 of the page's 64 keys, so the softmax needs one cross-lane step.
//  * Pages are staged through registers one page ahead into the other half
//    of a double buffer: one barrier a page.  Keys past the tile's last
//    token are staged as zeros (their cells may hold anything).
//  * O^T = V^T P^T with V read through the LDS transpose reads.  P goes in
//    as two bf16 parts (hi + lo), so the weights keep 16 significand bits;
//    both parts share the V fragments.
//  * Tied form (values are keys): one image of a page serves both products,
//    rows for the scores, transpose reads for the values; the swizzle keeps
//    both free of conflicts.  A key's factor and its distance bias join the
//    score in one multiply-add each.
//  * Window form: soft cap by one exponential and one reciprocal, the bias by
//    distance from LDS (a page whose every distance is beyond the table's
//    last adds a constant), kept first pages before the window's.
//  * Pages that no row of a wave sees are skipped by that wave; masks are
//    applied only on pages that a chunk edge or the diagonal crosses.

#include "lm.h"
#include "tile.h"
#include "attn.h"

namespace {

constexpr float LOG2E = 1.4426950408889634f;

DEVINL unsigned pack2(float a, float b) {
  return (unsigned)(unsigned short)cvt_bf16(a) |
         ((unsigned)(unsigned short)cvt_bf16(b) << 16);
}

DEVINL f32x16 mma32(bf16x8 a, bf16x8 b, f32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(
      __builtin_bit_cast(__attribute__((ext_vector_type(8))) __bf16, a),
      __builtin_bit_cast(__attribute__((ext_vector_type(8))) __bf16, b), c, 0,
      0, 0);
}

// B fragments (16 keys each) of 16 consecutive-by-lane P^T values
DEVINL void p_frags(const float* p, bf16x8 (&out)[2]) {
  #pragma unroll
  for (int s = 0; s < 2; ++s) {
    const unsigned ax = pack2(p[8 * s + 0], p[8 * s + 1]);
    const unsigned ay = pack2(p[8 * s + 2], p[8 * s + 3]);
    const unsigned bx = pack2(p[8 * s + 4], p[8 * s + 5]);
    const unsigned by = pack2(p[8 * s + 6], p[8 * s + 7]);
    auto rx = __builtin_amdgcn_permlane32_swap(ax, bx, false, false);
    auto ry = __builtin_amdgcn_permlane32_swap(ay, by, false, false);
    union { unsigned u[4]; bf16x8 v; } f;
    f.u[0] = rx[0]; f.u[1] = ry[0]; f.u[2] = rx[1]; f.u[3] = ry[1];
    out[s] = f.v;
  }
}

// Place of 8-column chunk cb of key j in a page's image.
template <int DK, bool TIED>
DEVINL int chunk_at(int j, int cb) {
  if constexpr (TIED) return tied_chunk<DK>(j, cb);
  else return cb ^ (j & 7);
}

constexpr int BIAS_LDS = 512;          // entries of a head's bias kept in LDS

// FORM 0: as stored; 1: with a bias by distance; 2: tied, with one; 3: window
template <int DK, int DV, int HPB, int FORM>
__global__ void __launch_bounds__(HPB * 128, 2)
attn_prefill_mfma_kernel(AttnArgs a, const int4* __restrict__ tiles,
                         int n_tiles) {
  constexpr int NT = HPB * 128;
  constexpr int NSL = DK / 16, NDT = DV / 32;
  constexpr bool TIED = FORM == 2, BIAS = FORM == 1 || FORM == 2;
  constexpr bool WIN = FORM == 3;
  static_assert(!TIED || DK == DV, "one image");
  constexpr int BUF = 64 * (DK + (TIED ? 0 : DV));  // K image + V tr-image
  constexpr int KC = 64 * DK / 8 / NT, VC = 64 * DV / 8 / NT;
  __shared__ __attribute__((aligned(16))) short lds[2 * BUF];
  __shared__ __attribute__((aligned(16))) float kfs[TIED ? 2 * 64 : 4];
  __shared__ float bias_s[WIN ? HPB * BIAS_LDS : 1];

  const int tid = threadIdx.x, l = tid & 63, wid = tid >> 6;
  const int lq = l & 31, half = l >> 5;
  int bx, by;
  xcd_tile_map(n_tiles, &bx, &by);
  bx = n_tiles - 1 - bx;               // a prompt's last tiles see most: first
  const int hg = a.H / a.G, nhc = hg / HPB;
  const int g = by / nhc;
  const int h = g * hg + (by % nhc) * HPB + (wid >> 1);
  const int4 t = tiles[bx];                    // first row, rows, pos0, slot
  const int row = 32 * (wid & 1) + lq;
  const int rowc = min(row, t.y - 1);
  const int ip = t.z + rowc;
  const int cs = first_seen(a, ip), keep = WIN ? a.keep : 0;

  bf16x8 qf[NSL];
  {
    const short* q = (const short*)a.qkv + (long)(t.x + rowc) * a.ld + (long)h * a.dim;
    #pragma unroll
    for (int s = 0; s < NSL; ++s) {
      const int c = 16 * s + 8 * half;
      qf[s] = c < a.dim ? *(const bf16x8*)(q + c) : bf16x8{};
    }
  }

  const int p_last = t.z + t.y - 1;
  const PageList pages(a, t.z, p_last);
  const int* tab = a.table + (long)t.w * a.max_pages;

  // this wave's rows: first and last position, and their chunk starts
  const int w0 = t.z + min(32 * (wid & 1), t.y - 1);
  const int w1 = t.z + min(32 * (wid & 1) + 31, t.y - 1);
  const bool w_any = 32 * (wid & 1) < t.y;
  const int wcs0 = first_seen(a, w0), wcs1 = first_seen(a, w1);

  bf16x8 kr[KC], vr[TIED ? 1 : VC];
  float kf = 0.f;
  const float scale2 = a.scale * LOG2E;
  auto stage_load = [&](int pg) {
    const long page = tab[pg];
    const short* kp = (const short*)a.kc + (page * a.G + g) * LM_PAGE * a.dim;
    const int left = p_last - pg * LM_PAGE;    // last valid key of the page
    #pragma unroll
    for (int i = 0; i < KC; ++i) {
      const int s = i * NT + tid, j = s / (DK / 8), c = (s % (DK / 8)) * 8;
      kr[i] = c < a.dim && (!TIED || j <= left)
                  ? *(const bf16x8*)(kp + (long)j * a.dim + c) : bf16x8{};
    }
    if constexpr (TIED) {
      if (tid < 64) kf = tid <= left ? a.ks[page * LM_PAGE + tid] * scale2 : 0.f;
    } else {
      const short* vp = (const short*)a.vc + (page * a.G + g) * LM_PAGE * a.vdim;
      #pragma unroll
      for (int i = 0; i < VC; ++i) {
        const int s = i * NT + tid, j = s / (DV / 8), c = (s % (DV / 8)) * 8;
        vr[i] = c < a.vdim && j <= left
                    ? *(const bf16x8*)(vp + (long)j * a.vdim + c) : bf16x8{};
      }
    }
  };
  auto stage_write = [&](int buf) {
    short* kd = lds + buf * BUF;
    short* vd = kd + 64 * DK;
    #pragma unroll
    for (int i = 0; i < KC; ++i) {
      const int s = i * NT + tid, j = s / (DK / 8), cb = s % (DK / 8);
      *(bf16x8*)(kd + j * DK + chunk_at<DK, TIED>(j, cb) * 8) = kr[i];
    }
    if constexpr (TIED) {
      if (tid < 64) kfs[buf * 64 + tid] = kf;
    } else {
      #pragma unroll
      for (int i = 0; i < VC; ++i) {
        const int s = i * NT + tid, j = s / (DV / 8), c = (s % (DV / 8)) * 8;
        *(bf16x8*)(vd + ((j >> 2) * (DV / 16) + (c >> 4)) * 64 + (j & 3) * 16 +
                   (c & 15)) = vr[i];
      }
    }
  };
  // transpose reads: this lane's 8 bytes of a 4-key x 16-column subtile
  const unsigned tr0 = lds_byte_off(lds + 64 * DK) + 128u * (lq >> 4) +
                       ((l & 15) >> 2) * 32 + (l & 3) * 8 +
                       (half ? 128u * 2 * (DV / 16) : 0);
  // the same out of the tied image: row 8 * half + r of a 16-key step,
  // r = 0..3, and the chunk that chunk_at gives for it; steps, quads and
  // column tiles only flip bits of the chunk
  const int tr_r = (l & 15) >> 2;
  const unsigned tk0 = lds_byte_off(lds) + (8 * half + tr_r) * (DK * 2) + (l & 1) * 8;
  const unsigned tkc = chunk_at<DK, true>(8 * half + tr_r,
                                          2 * (lq >> 4) + ((l & 3) >> 1)) * 16;

  const float slope2 = BIAS && a.slopes ? a.slopes[h] * LOG2E : 0.f;
  float m_run = a.has_sink ? sink_score<false>(a, h) * LOG2E : -1e30f;
  float l_run = a.has_sink ? 1.f : 0.f;
  f32x16 o[NDT];
  #pragma unroll
  for (int i = 0; i < NDT; ++i) o[i] = {};

  // window form: this head's bias in base 2
  const int n_bias = WIN ? a.n_bias : 0;
  const bool bias_lds = n_bias <= BIAS_LDS;
  const float* bias_g = nullptr;
  const float* bias_h = bias_s + (wid >> 1) * BIAS_LDS;
  float bias_far = 0.f;
  if constexpr (WIN) {
    bias_g = a.bias + (long)h * n_bias;
    bias_far = bias_g[n_bias - 1] * LOG2E;
    if (bias_lds)
      for (int i = tid % 128; i < n_bias; i += 128)
        bias_s[(wid >> 1) * BIAS_LDS + i] = bias_g[i] * LOG2E;
  }
  const SoftCap cap(a, LOG2E);

  stage_load(pages[0]);
  stage_write(0);
  __syncthreads();
  int cur = 0;
  for (int it = 0; it < pages.n; ++it) {
    const int pg = pages[it];
    if (it + 1 < pages.n) stage_load(pages[it + 1]);
    const int j0 = pg * LM_PAGE;
    if (w_any && j0 <= w1 && (j0 + LM_PAGE > wcs0 || j0 < keep)) {
      const short* kimg = lds + cur * BUF;
      f32x16 s[2];
      s[0] = {};
      s[1] = {};
      #pragma unroll
      for (int sub = 0; sub < 2; ++sub) {
        const int kr_ = sub * 32 + lq;
        #pragma unroll
        for (int i = 0; i < NSL; ++i)
          s[sub] = mma32(*(const bf16x8*)(kimg + kr_ * DK +
                                          chunk_at<DK, TIED>(kr_, 2 * i + half) * 8),
                         qf[i], s[sub]);
      }
      const bool edge = j0 + LM_PAGE - 1 > w0 || j0 < wcs1;
      float mt = -1e30f;
      const float d0 = slope2 * (float)(j0 + 4 * half - ip);
      if constexpr (WIN) {
        const int last = n_bias - 1, dist = ip - j0 - 4 * half;
        const bool far = w0 - j0 - (LM_PAGE - 1) >= last;     // of all rows
        float most = 0.f;
        #pragma unroll
        for (int sub = 0; sub < 2; ++sub)
          #pragma unroll
          for (int r = 0; r < 16; ++r) most = fmaxf(most, fabsf(s[sub][r]));
        const bool small = cap.small(most);
        // both are uniform in the wave
        auto scores = [&](auto bias) {
          #pragma unroll
          for (int sub = 0; sub < 2; ++sub)
            #pragma unroll
            for (int r = 0; r < 16; ++r) {
              const float b = bias(sub * 32 + (r & 3) + 8 * (r >> 2));
              s[sub][r] = small ? cap.near(s[sub][r], b) : cap.any(s[sub][r], b);
            }
        };
        if (far) {
          if (small) {
            #pragma unroll
            for (int sub = 0; sub < 2; ++sub)
              #pragma unroll
              for (int r = 0; r < 16; ++r) s[sub][r] = cap.near(s[sub][r], bias_far);
          } else {
            #pragma unroll
            for (int sub = 0; sub < 2; ++sub)
              #pragma unroll
              for (int r = 0; r < 16; ++r) s[sub][r] = cap.any(s[sub][r], bias_far);
          }
        } else if (bias_lds) {
          scores([&](int j) { return bias_h[min(max(dist - j, 0), last)]; });
        } else {
          scores([&](int j) { return bias_g[min(max(dist - j, 0), last)] * LOG2E; });
        }
      }
      #pragma unroll
      for (int sub = 0; sub < 2; ++sub)
        #pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int jr = sub * 32 + (r & 3) + 8 * (r >> 2);
          float x = s[sub][r];
          if constexpr (TIED) x *= kfs[cur * 64 + jr + 4 * half];
          else if constexpr (!WIN) x *= scale2;
          if constexpr (BIAS) x += fmaf(slope2, (float)jr, d0);
          if (edge) {
            const int j = j0 + jr + 4 * half;
            x = j <= ip && (j >= cs || (WIN && j < keep)) ? x : -1e30f;
          }
          s[sub][r] = x;
          mt = fmaxf(mt, x);
        }
      mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
      // a row that has seen no key of its own yet collects finite junk
      // here; its first own key sets m_run and wipes it (alpha = 0)
      if (__any(mt > m_run)) {
        const float mn = fmaxf(m_run, mt);
        const float al = __builtin_amdgcn_exp2f(m_run - mn);
        m_run = mn;
        l_run *= al;
        #pragma unroll
        for (int i = 0; i < NDT; ++i)
          #pragma unroll
          for (int r = 0; r < 16; ++r) o[i][r] *= al;
      }
      float ps = 0.f;
      #pragma unroll
      for (int sub = 0; sub < 2; ++sub)
        #pragma unroll
        for (int r = 0; r < 16; ++r) {
          s[sub][r] = __builtin_amdgcn_exp2f(s[sub][r] - m_run);
          ps += s[sub][r];
        }
      l_run += ps + __shfl_xor(ps, 32, 64);

      #pragma unroll
      for (int sub = 0; sub < 2; ++sub) {
        float p[16], q[16];
        #pragma unroll
        for (int r = 0; r < 16; ++r) p[r] = s[sub][r];
        bf16x8 hi[2], lo[2];
        p_frags(p, hi);
        #pragma unroll
        for (int r = 0; r < 16; ++r) q[r] = p[r] - bf2f(cvt_bf16(p[r]));
        p_frags(q, lo);
        const unsigned base = tr0 + (unsigned)cur * (BUF * 2) + (unsigned)sub * (32u * DV * 2);
        #pragma unroll
        for (int t2 = 0; t2 < NDT; t2 += 2) {
          auto addr = [&](int tt, int ss) {
            return base + 128u * (unsigned)((4 * ss) * (DV / 16) + 2 * tt);
          };
          const unsigned qs = 128u * (DV / 16);
          // column tile tt, 16-key step ss, quad q of it (tied image)
          auto tied = [&](int tt, int ss, int q) {
            const unsigned flip = (DK == 64 ? q : 8 * q) ^ (4 * tt);
            return tk0 + (unsigned)cur * (BUF * 2) +
                   (unsigned)(32 * sub + 16 * ss + 4 * q) * (DK * 2) +
                   (tkc ^ (flip * 16));
          };
          bf16x8_quad v;
          if constexpr (TIED)
            v = tr_read_quad(tied(t2, 0, 0), tied(t2, 0, 1), tied(t2, 1, 0),
                             tied(t2, 1, 1), tied(t2 + 1, 0, 0),
                             tied(t2 + 1, 0, 1), tied(t2 + 1, 1, 0),
                             tied(t2 + 1, 1, 1));
          else
            v = tr_read_quad(
              addr(t2, 0), addr(t2, 0) + qs, addr(t2, 1), addr(t2, 1) + qs,
              addr(t2 + 1, 0), addr(t2 + 1, 0) + qs, addr(t2 + 1, 1),
              addr(t2 + 1, 1) + qs);
          o[t2] = mma32(v.f[0], hi[0], o[t2]);
          o[t2 + 1] = mma32(v.f[2], hi[0], o[t2 + 1]);
          o[t2] = mma32(v.f[1], hi[1], o[t2]);
          o[t2 + 1] = mma32(v.f[3], hi[1], o[t2 + 1]);
          o[t2] = mma32(v.f[0], lo[0], o[t2]);
          o[t2 + 1] = mma32(v.f[2], lo[0], o[t2 + 1]);
          o[t2] = mma32(v.f[1], lo[1], o[t2]);
          o[t2 + 1] = mma32(v.f[3], lo[1], o[t2 + 1]);
        }
      }
    }
    // the other buffer's readers passed the barrier of the last page
    if (it + 1 < pages.n) stage_write(cur ^ 1);
    __syncthreads();
    cur ^= 1;
  }

  if (row < t.y) {
    const float inv = l_run > 0.f ? a.out_scale / l_run : 0.f;
    short* dst = (short*)a.out + (long)(t.x + row) * a.ldo + (long)h * a.vdim;
    const short* gate = a.gate ? (const short*)a.gate + (long)(t.x + row) * a.ld +
                                     (long)h * a.vdim : nullptr;
    #pragma unroll
    for (int i = 0; i < NDT; ++i)
      #pragma unroll
      for (int rq = 0; rq < 4; ++rq) {
        const int d = 32 * i + 8 * rq + 4 * half;
        if (d >= a.vdim) continue;
        bf16x4 pk, gt{};
        if (gate) gt = *(const bf16x4*)(gate + d);
        #pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float y = o[i][rq * 4 + j] * inv;
          pk[j] = cvt_bf16(gate ? y * sigmoid(bf2f(gt[j])) : y);
        }
        *(bf16x4*)(dst + d) = pk;
      }
  }
}

template <int DK, int DV, int FORM>
void launch(const AttnArgs& a, const int4* tiles, int n, hipStream_t st) {
  const int hg = a.H / a.G;
  #define AM_GO(HPB)                                                           \
    hipLaunchKernelGGL((attn_prefill_mfma_kernel<DK, DV, HPB, FORM>),          \
                       dim3((unsigned)((long)n * a.G * (hg / HPB))),           \
                       dim3(HPB * 128), 0, st, a, tiles, n)
  if (hg % 4 == 0) AM_GO(4);
  else if (hg % 2 == 0) AM_GO(2);
  else AM_GO(1);
  #undef AM_GO
}

template <int DK, int DV>
void pick_form(const AttnArgs& a, const int4* tiles, int n, hipStream_t st) {
  if (a.bias) launch<DK, DV, 3>(a, tiles, n, st);
  else if (a.slopes) launch<DK, DV, 1>(a, tiles, n, st);
  else launch<DK, DV, 0>(a, tiles, n, st);
}

}  // namespace

bool lm_attn_mfma_ok(const AttnArgs& a) {
  // rows of out that vectors can be stored to
  return a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= 128 && a.vdim <= 128 &&
         a.ldo % 4 == 0 && (size_t)a.out % 8 == 0;
}

void lm_attn_prefill_mfma(const AttnArgs& a, const int4* tiles, int n_tiles,
                          hipStream_t st) {
  if (a.ks) {
    if (a.dim <= 64) launch<64, 64, 2>(a, tiles, n_tiles, st);
    else launch<128, 128, 2>(a, tiles, n_tiles, st);
  } else if (a.dim <= 64) {
    if (a.vdim <= 64) pick_form<64, 64>(a, tiles, n_tiles, st);
    else pick_form<64, 128>(a, tiles, n_tiles, st);
  } else {
    if (a.vdim <= 64) pick_form<128, 64>(a, tiles, n_tiles, st);
    else pick_form<128, 128>(a, tiles, n_tiles, st);
  }
}
