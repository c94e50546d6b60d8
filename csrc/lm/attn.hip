// Prompt attention over a paged cache: grouped heads, chunked causal mask,
// optional sink in the softmax denominator, separate key and value widths,
// or values that are the keys (tied form), a bias by distance, an output gate;
// or a sliding window beside which the first tokens stay visible, soft-capped
// scores and a learned bias by distance (window form).
//
// The kv loop walks cache pages (64 keys), so a tile of keys is one
// contiguous block per kv head whatever the prompt's cut.  Row i of a tile
// sits at absolute position pos0 + i and sees keys from the start of its
// own chunk to itself; only pages between the first row's chunk start and
// the last row are visited.
//
// Scores, the running maximum and sum and the weights are float.  In bf16
// mode the weights enter the value product as two bf16 parts, which keeps
// 16 significand bits of them.

#include "lm.h"
#include "tile.h"
#include "attn.h"

#include <type_traits>

namespace {

constexpr float LOG2E = 1.4426950408889634f;

// One lane group (LPV lanes, 8 elements each) per (row, head) vector: RMS
// norm over `dim` for q heads (in place; left out if q has none) and k heads
// (into the cache), plain copy for v heads or (v_norm) a norm without weights.
template <bool F32, int LPV>
__global__ void __launch_bounds__(256)
attn_prep_kernel(AttnArgs a, const int* __restrict__ pos,
                 const int* __restrict__ slot, int row0, int n) {
  using N = Num<F32>;
  using E = typename N::E;
  const int h0 = a.qw ? 0 : a.H, heads = a.H + 2 * a.G - h0;
  const long unit = ((long)blockIdx.x * 256 + threadIdx.x) / LPV;
  if (unit >= (long)n * heads) return;
  const int c = (threadIdx.x % LPV) * 8;
  const int row = row0 + (int)(unit / heads);
  const int hd = h0 + (int)(unit % heads);
  const int s = slot[row];
  if (s < 0) return;
  const int p = pos[row];
  const bool aligned = a.dim % 8 == 0 && a.vdim % 8 == 0;
  const bool is_v = hd >= a.H + a.G;
  const int len = is_v ? a.vdim : a.dim;
  E* src = (E*)a.qkv + (long)row * a.ld +
           (is_v ? (long)(a.H + a.G) * a.dim + (long)(hd - a.H - a.G) * a.vdim
                 : (long)hd * a.dim);
  E* dst = src;
  if (hd >= a.H) {
    const int g = is_v ? hd - a.H - a.G : hd - a.H;
    const long page = a.table[(long)s * a.max_pages + p / LM_PAGE];
    dst = (E*)(is_v ? a.vc : a.kc) +
          ((page * a.G + g) * LM_PAGE + p % LM_PAGE) * len;
  }
  float v[8];
  load8<F32>(src + c, len - c, aligned, v);
  const E* w = (const E*)(is_v ? nullptr : hd < a.H ? a.qw : a.kw);
  float q = 0.f;
  #pragma unroll
  for (int i = 0; i < 8; ++i) q += v[i] * v[i];
  q = group_sum<LPV>(q);
  if (w) {
    const float inv = 1.0f / sqrtf(q / (float)a.dim + a.eps);
    float wv[8];
    load8<F32>(w + c, len - c, aligned, wv);
    #pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= inv * wv[i];
  } else if (is_v && a.v_norm) {
    const float inv = 1.0f / sqrtf(q / (float)a.vdim + a.eps);
    #pragma unroll
    for (int i = 0; i < 8; ++i) v[i] *= inv;
  }
  store8<F32>(dst + c, len - c, aligned, v);
}

// Tied form, one block per row: q by its root mean square over all heads,
// its weights, the temperature of its position and the key weights (which a
// score takes from either side); k as it is into the cache, beside the
// factor that norms it.
template <bool F32, int VEC>
__global__ void __launch_bounds__(256)
attn_prep_tied_kernel(AttnArgs a, const int* __restrict__ pos,
                      const int* __restrict__ slot, int row0) {
  using N = Num<F32>;
  using E = typename N::E;
  __shared__ float red[2][4];
  const int row = row0 + blockIdx.x, tid = threadIdx.x;
  const int s = slot[row];
  if (s < 0) return;
  const int p = pos[row];
  const int nq = a.H * a.dim, nk = a.G * a.dim, hg = a.H / a.G;
  E* q = (E*)a.qkv + (long)row * a.ld;
  const E* k = q + nq;
  auto get = [&](const E* src, float (&v)[VEC]) {
    if constexpr (VEC == 8) load8<F32>(src, 8, true, v);
    else v[0] = N::up(src[0]);
  };
  float sq = 0.f, sk = 0.f, v[VEC];
  for (int e = tid * VEC; e < nq; e += 256 * VEC) {
    get(q + e, v);
    #pragma unroll
    for (int i = 0; i < VEC; ++i) sq += v[i] * v[i];
  }
  const long cell = (long)a.table[(long)s * a.max_pages + p / LM_PAGE];
  for (int e = tid * VEC; e < nk; e += 256 * VEC) {
    get(k + e, v);
    #pragma unroll
    for (int i = 0; i < VEC; ++i) sk += v[i] * v[i];
    E* dst = (E*)a.kc + ((cell * a.G + e / a.dim) * LM_PAGE + p % LM_PAGE) * a.dim +
             e % a.dim;
    if constexpr (VEC == 8) store8<F32>(dst, 8, true, v);
    else dst[0] = N::down(v[0]);
  }
  sq = group_sum<64>(sq);
  sk = group_sum<64>(sk);
  if ((tid & 63) == 0) {
    red[0][tid >> 6] = sq;
    red[1][tid >> 6] = sk;
  }
  __syncthreads();
  sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
  sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  if (tid == 0)
    a.ks[cell * LM_PAGE + p % LM_PAGE] = 1.0f / sqrtf(sk / (float)nk + a.eps);
  const float inv = temperature(a, p) / sqrtf(sq / (float)nq + a.eps);
  for (int e = tid * VEC; e < nq; e += 256 * VEC) {
    float w[VEC], u[VEC];
    get(q + e, v);
    get((const E*)a.qw + e, w);
    get((const E*)a.kw + (e / a.dim / hg) * a.dim + e % a.dim, u);
    #pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] *= inv * w[i] * u[i];
    if constexpr (VEC == 8) store8<F32>(q + e, 8, true, v);
    else q[e] = N::down(v[0]);
  }
}

// 4 waves, 16 query rows each; one query head per block.
template <bool F32, int DK, int DV>
__global__ void __launch_bounds__(256)
attn_prefill_kernel(AttnArgs a, const int4* __restrict__ tiles) {
  using N = Num<F32>;
  using E = typename N::E;
  constexpr int LDK = DK + N::PAD;
  constexpr int LDJ = LM_PAGE + N::PAD;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  E* Ks = (E*)smem;                       // [64][LDK]
  E* Vt = Ks + LM_PAGE * LDK;             // [DV][LDJ]  values, transposed
  E* Pb = Vt + DV * LDJ;                  // [PARTS][64][LDJ]
  float* Kf = (float*)(Pb + Split<F32>::PARTS * LM_TILE * LDJ);  // [64]
  const Split<F32> P{Pb, Pb + LM_TILE * LDJ};

  const int4 t = tiles[blockIdx.x];       // first row, rows, pos0, slot
  const int h = blockIdx.y, g = h / (a.H / a.G);
  const int tid = threadIdx.x, w = tid >> 6, l = tid & 63;
  const int lr = l & 15, lg = l >> 4;
  const bool aligned = a.dim % 8 == 0 && a.vdim % 8 == 0;

  // this wave's 16 q rows as A fragments
  typename N::Frag qf[DK / 32];
  {
    const int r = 16 * w + lr;
    const E* qrow = (const E*)a.qkv + (long)(t.x + min(r, t.y - 1)) * a.ld + (long)h * a.dim;
    #pragma unroll
    for (int kb = 0; kb < DK / 32; ++kb) {
      float v[8];
      const int c = kb * 32 + lg * 8;
      load8<F32>(qrow + c, a.dim - c, aligned, v);
      #pragma unroll
      for (int i = 0; i < 8; ++i) {
        if constexpr (F32) qf[kb].v[i] = v[i];
        else qf[kb][i] = N::down(v[i]);
      }
    }
  }

  const float scale2 = a.scale * LOG2E;   // softmax in base 2
  const float slope2 = a.slopes ? a.slopes[h] * LOG2E : 0.f;
  const bool tied = a.ks != nullptr;
  int cs[4], ip[4];                       // chunk start, position per row
  float m[4], lsum[4];
  f32x4 o[DV / 16];
  #pragma unroll
  for (int i = 0; i < DV / 16; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = 16 * w + 4 * lg + r;
    ip[r] = t.z + min(row, t.y - 1);
    cs[r] = first_seen(a, ip[r]);
    m[r] = a.has_sink ? sink_score<F32>(a, h) * LOG2E : -1e30f;
    lsum[r] = a.has_sink ? 1.f : 0.f;
  }

  const int p_last = t.z + t.y - 1;
  const PageList pages(a, t.z, p_last);
  const int* tab = a.table + (long)t.w * a.max_pages;
  const float* bias = a.bias ? a.bias + (long)h * a.n_bias : nullptr;
  for (int it = 0; it < pages.n; ++it) {
    const int pg = pages[it];
    const long page = tab[pg];
    const E* kp = (const E*)a.kc + (page * a.G + g) * LM_PAGE * a.dim;
    const E* vp = (const E*)a.vc + (page * a.G + g) * LM_PAGE * a.vdim;
    const int j0 = pg * LM_PAGE;
    __syncthreads();                      // the last tile's reads are over
    if (tid < LM_PAGE)
      Kf[tid] = tied ? (j0 + tid <= p_last ? a.ks[page * LM_PAGE + tid] : 0.f) : 1.f;
    for (int u = tid; u < LM_PAGE * (DK / 8); u += 256) {
      const int j = u / (DK / 8), c = (u % (DK / 8)) * 8;
      float v[8];
      const bool ok = j0 + j <= p_last;
      load8<F32>(kp + (long)j * a.dim + c, ok ? a.dim - c : 0, aligned, v);
      #pragma unroll
      for (int i = 0; i < 8; ++i) Ks[j * LDK + c + i] = N::down(v[i]);
    }
    for (int u = tid; u < LM_PAGE * (DV / 8); u += 256) {
      const int j = u % LM_PAGE, c = (u / LM_PAGE) * 8;
      float v[8];
      const bool ok = j0 + j <= p_last;
      load8<F32>(vp + (long)j * a.vdim + c, ok ? a.vdim - c : 0, aligned, v);
      #pragma unroll
      for (int i = 0; i < 8; ++i) Vt[(c + i) * LDJ + j] = N::down(v[i]);
    }
    __syncthreads();

    f32x4 s[4];
    #pragma unroll
    for (int ct = 0; ct < 4; ++ct) {
      s[ct] = f32x4{0.f, 0.f, 0.f, 0.f};
      #pragma unroll
      for (int kb = 0; kb < DK / 32; ++kb)
        s[ct] = N::mma(qf[kb], N::load(Ks + (ct * 16 + lr) * LDK, kb * 32 + lg * 8), s[ct]);
    }
    float mx[4] = {-1e30f, -1e30f, -1e30f, -1e30f};
    #pragma unroll
    for (int ct = 0; ct < 4; ++ct)
      #pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = j0 + ct * 16 + lr;
        const bool see = j <= ip[r] && (j >= cs[r] || j < a.keep);
        float x = s[ct][r];
        if (bias) {
          x *= a.scale;
          if (a.softcap > 0.f) x = a.softcap * tanhf(x / a.softcap);
          x = (x + bias[min(max(ip[r] - j, 0), a.n_bias - 1)]) * LOG2E;
        } else {
          x = x * (scale2 * Kf[ct * 16 + lr]) - slope2 * (float)(ip[r] - j);
        }
        s[ct][r] = see ? x : -1e30f;
        mx[r] = fmaxf(mx[r], s[ct][r]);
      }
    #pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float mn = fmaxf(m[r], max16(mx[r]));
      const float al = exp2f(m[r] - mn);
      m[r] = mn;
      float ps = 0.f;
      #pragma unroll
      for (int ct = 0; ct < 4; ++ct) {
        // a row that has seen no key yet has mn = -1e30: its weights are 0
        const float e = s[ct][r] > -1e29f ? exp2f(s[ct][r] - mn) : 0.f;
        ps += e;
        P.put((16 * w + 4 * lg + r) * LDJ + ct * 16 + lr, e);
      }
      lsum[r] = lsum[r] * al + sum16(ps);
      #pragma unroll
      for (int i = 0; i < DV / 16; ++i) o[i][r] *= al;
    }
    // P rows are written and read by the same wave; order its LDS ops
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    #pragma unroll
    for (int kb = 0; kb < LM_PAGE / 32; ++kb) {
      const auto pf = P.load((16 * w + lr) * LDJ, kb * 32 + lg * 8);
      #pragma unroll
      for (int i = 0; i < DV / 16; ++i)
        o[i] = mma_sp<F32>(pf, N::load(Vt + (i * 16 + lr) * LDJ, kb * 32 + lg * 8), o[i]);
    }
  }

  #pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = 16 * w + 4 * lg + r;
    if (row >= t.y) continue;
    const float inv = lsum[r] > 0.f ? a.out_scale / lsum[r] : 0.f;
    E* dst = (E*)a.out + (long)(t.x + row) * a.ldo + (long)h * a.vdim;
    const E* gate = a.gate ? (const E*)a.gate + (long)(t.x + row) * a.ld +
                                 (long)h * a.vdim : nullptr;
    #pragma unroll
    for (int i = 0; i < DV / 16; ++i) {
      const int c = i * 16 + lr;
      if (c < a.vdim)
        dst[c] = N::down(o[i][r] * inv * (gate ? sigmoid(N::up(gate[c])) : 1.f));
    }
  }
}

template <bool F32, int DK, int DV>
void launch_prefill(const AttnArgs& a, const int4* tiles, int n_tiles,
                    hipStream_t st) {
  using N = Num<F32>;
  constexpr int LDJ = LM_PAGE + N::PAD;
  constexpr size_t lds = sizeof(typename N::E) *
      (LM_PAGE * (DK + N::PAD) + DV * LDJ + Split<F32>::PARTS * LM_TILE * LDJ) +
      sizeof(float) * LM_PAGE;
  static_assert(lds <= 160 * 1024, "exceeds the CU's LDS");
  static const hipError_t attr = hipFuncSetAttribute(
      (const void*)attn_prefill_kernel<F32, DK, DV>,
      hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
  (void)attr;
  hipLaunchKernelGGL((attn_prefill_kernel<F32, DK, DV>), dim3(n_tiles, a.H),
                     dim3(256), lds, st, a, tiles);
}

template <bool F32, int DK>
void pick_dv(const AttnArgs& a, const int4* tiles, int n, hipStream_t st) {
  if (a.vdim <= 64) launch_prefill<F32, DK, 64>(a, tiles, n, st);
  else if (a.vdim <= 128) launch_prefill<F32, DK, 128>(a, tiles, n, st);
  else launch_prefill<F32, DK, 256>(a, tiles, n, st);
}

template <bool F32>
void pick_dk(const AttnArgs& a, const int4* tiles, int n, hipStream_t st) {
  if (a.dim <= 64) pick_dv<F32, 64>(a, tiles, n, st);
  else if (a.dim <= 128) pick_dv<F32, 128>(a, tiles, n, st);
  else pick_dv<F32, 256>(a, tiles, n, st);
}

}  // namespace

namespace {
template <bool F32>
void run_prep(const AttnArgs& a, const int* pos, const int* slot, int row0,
              int n, hipStream_t st) {
  const long units = (long)n * ((a.qw ? a.H : 0) + 2 * a.G);
  const int d = std::max(a.dim, a.vdim);
  #define AP_GO(LPV)                                                           \
    hipLaunchKernelGGL((attn_prep_kernel<F32, LPV>),                           \
                       dim3((unsigned)((units * LPV + 255) / 256)), dim3(256), \
                       0, st, a, pos, slot, row0, n)
  if (d <= 32) AP_GO(4);
  else if (d <= 64) AP_GO(8);
  else if (d <= 128) AP_GO(16);
  else AP_GO(32);
  #undef AP_GO
}
}  // namespace

void lm_attn_prep(const AttnArgs& a, const int* pos, const int* slot, int row0,
                  int n, bool f32, hipStream_t stream) {
  if (n <= 0) return;
  if (a.ks) {
    const bool v8 = a.dim % 8 == 0;
    #define TP_GO(F, V)                                                        \
      hipLaunchKernelGGL((attn_prep_tied_kernel<F, V>), dim3(n), dim3(256), 0, \
                         stream, a, pos, slot, row0)
    if (f32) { if (v8) TP_GO(true, 8); else TP_GO(true, 1); }
    else { if (v8) TP_GO(false, 8); else TP_GO(false, 1); }
    #undef TP_GO
    return;
  }
  if (f32) run_prep<true>(a, pos, slot, row0, n, stream);
  else run_prep<false>(a, pos, slot, row0, n, stream);
}

void lm_attn_prefill(const AttnArgs& a, const int4* tiles, int n_tiles,
                     bool f32, hipStream_t stream) {
  if (n_tiles <= 0) return;
  if (f32) pick_dk<true>(a, tiles, n_tiles, stream);
  else if (lm_attn_mfma_ok(a)) lm_attn_prefill_mfma(a, tiles, n_tiles, stream);
  else pick_dk<false>(a, tiles, n_tiles, stream);
}
