// Launchers of the mixer-stack serving kernels.  Raw pointers only: the
// shapes were checked by the binding layer (ext.cpp) before these run.
//
// Conventions shared by all of them:
//   f32      true: activations, weights and caches are float; false: bf16
//   table    int [slots][max_pages], page ids of a sequence in order
//   page     64 tokens; key caches are [page][kv_heads][64][dim]
//   tiles    int4 {first row, rows (<= 64), position of the first row, slot}
//            one entry per up-to-64 consecutive prompt tokens of a sequence
//   slots    int [rows]; a negative slot marks a row that must touch nothing
#pragma once

#include <hip/hip_runtime.h>

constexpr int LM_PAGE = 64;   // tokens per cache page
constexpr int LM_TILE = 64;   // prompt tokens per tile

// ---- norm.hip
// w null: no norm; alpha null: layer or RMS norm, else tanh(alpha x) w + b
struct LmNorm {
  const void* w;
  const void* b;      // or null
  const void* alpha;  // one element, or null
  bool rms;
  bool one;           // w is one element, for all columns
};
// a sublayer's output: y [T][W] (or null), or with weights w [T][n] the
// weighted sum over n of y [T][n][W]
struct LmSum {
  const void* y;
  const float* w;
  int n;
};
// ptab: learned positions [n_pos][W] to add at pos [T], or null
void lm_embed_norm(const long* tokens, const void* embed, const int* pos,
                   const void* ptab, int n_pos, float* x, LmNorm nxt, void* h,
                   int T, int W, long vocab, float eps, bool f32,
                   hipStream_t stream);
void lm_residual_norm(float* x, LmSum y, LmNorm post, float mult,
                      LmNorm nxt, void* h, const int* rows, int T, int W,
                      float eps, bool store_x, bool f32, hipStream_t stream);
// x as above (y may be null), h rows [x | embed[token]]
void lm_residual_concat(float* x, LmSum y, LmNorm post, float mult,
                        const long* tokens, const void* embed, void* h, int T,
                        int W, long vocab, float eps, bool f32,
                        hipStream_t stream);
// x <- y + step, h <- norm of it
void lm_replace_norm(float* x, const void* y, bool y_f32, const void* step,
                     LmNorm nxt, void* h, int T, int W, float eps, bool f32,
                     hipStream_t stream);
void lm_gelu_erf(const void* in, void* out, long n, bool f32,
                 hipStream_t stream);
// rows [g | u], each n wide: gelu(g) u, or with clamps
// g' sigmoid(alpha g') (u' + shift)
constexpr int LM_GELU_TANH = 0, LM_CLAMPED = 1;
void lm_gated_act(const void* in, void* out, long rows, int n, int act,
                  float limit, float alpha, float shift, bool f32,
                  hipStream_t stream);
void lm_softcap(const void* in, float* out, long n, float cap, bool f32,
                hipStream_t stream);
// RMS norm of each of a row's `parts` spans of n elements, times w and, if
// there is a gate (rows of stride ldg), its sigmoid
void lm_grouped_rms(const void* y, const void* w, const void* gate, long ldg,
                    void* out, long rows, int parts, int n, float eps, bool f32,
                    hipStream_t stream);

// ---- stream.hip: the start of a stream, and norms that look a token back
struct RaggedRows {   // where the rows of a batch lie (see StepPlan)
  const int* pos;
  const int* slot;
  const int4* tiles;  // first row, rows, position, slot
  const int4* seqs;   // first tile, tiles, position, slot
  int n_seqs, n_dec, T;
};
struct EmbedArgs {
  const long* tokens;
  const void* embed;
  long vocab;
  const double* rates;  // [(W + 1) / 2] turns per position, or null
  const void* pairs;    // [buckets + 1][W] or null
  long buckets, mul_prev, mul_cur;
  long* last;           // [slots] the token before
  float* x;
  int W;
};
void lm_stream_embed(const EmbedArgs& a, const RaggedRows& r, bool f32,
                     hipStream_t stream);
struct ShiftArgs {
  const float* x;
  LmSum y;
  float mult;
  const float* add;     // [T][W] or null
  const void* step;     // [W] or null
  LmNorm nxt;           // no alpha
  const void* shift;    // [W] or null
  float* state;         // [slots][W], with shift
  float* xo;            // x + mult * y + add + step; not x
  void* h;              // its norm, blended with the row before
  int W;
  float eps;
};
void lm_shift_norm(const ShiftArgs& a, const RaggedRows& r, bool f32,
                   hipStream_t stream);

// ---- attn.hip / attn_decode.hip
struct AttnArgs {
  void* qkv;          // rows of [heads*dim | kv_heads*dim | kv_heads*vdim],
                      // tied form [heads*dim | kv_heads*dim | heads*dim (gate)]
  long ld;            // row stride of qkv (elements)
  void* kc;
  void* vc;
  void* out;          // rows of [heads*vdim]
  const void* qw;     // per-head RMS weights or null
  const void* kw;
  const void* sink;   // [heads] or null: every head's is sink0
  float sink0;
  bool has_sink;
  long ldo;           // row stride of out
  float out_scale;    // multiplies out
  bool v_norm;        // each head's value over its root mean square
  // window form (bias not null): `size` is a sliding window, beside which the
  // first `keep` tokens stay visible; softcap * tanh(score / softcap)
  // (softcap 0: the score), then bias[h][min(distance, n_bias - 1)]
  const float* bias;  // [heads][n_bias]
  int n_bias;
  int keep;
  float softcap;
  const float* slopes;  // [heads] taken off a score per step of distance, or null
  // tied form (ks not null): the cached rows are the keys before their norm
  // and the values as well; token j's score takes the factor ks[j].  Norms
  // go over a whole row of q and of k, qw is [heads*dim], kw [kv_heads*dim];
  // q also takes 1 + t_coef ln(floor((p + 1) / t_every) + 1) at position p.
  float* ks;          // [pages][64]
  const void* gate;   // rows of stride ld: sigmoid of it multiplies out, or null
  float t_coef;
  int t_every;        // 0: no such factor
  const int* table;
  int max_pages;
  int H, G, dim, vdim;
  int size;           // chunk or window length in tokens; 0 = plain causal
  float scale;
  float eps;
};
// rows [row0, row0 + n): norm q in place, norm k into the cache, copy v
void lm_attn_prep(const AttnArgs& a, const int* pos, const int* slot, int row0,
                  int n, bool f32, hipStream_t stream);
void lm_attn_prefill(const AttnArgs& a, const int4* tiles, int n_tiles,
                     bool f32, hipStream_t stream);
// bf16, head sizes that are multiples of 8 up to 128
bool lm_attn_mfma_ok(const AttnArgs& a);
void lm_attn_prefill_mfma(const AttnArgs& a, const int4* tiles, int n_tiles,
                          hipStream_t stream);
// bf16, tied form: up to 16 heads a block instead of 4
bool lm_attn_decode_tied_mfma(const AttnArgs& a);
// rows [0, R), one token each; ws holds R*H*nsplit*(vdim+2) floats
void lm_attn_decode(const AttnArgs& a, const int* pos, const int* slot, int R,
                    int nsplit, float* ws, bool f32, hipStream_t stream);

// ---- retention.hip
struct RetArgs {
  const void* qkvg;   // rows of [H*dk | H*dk | H*dv | H*dv]
  long ld;
  float* state;       // [slots][H][dv][dk]
  void* out;          // rows of [H*dv]
  const float* pows;  // [H][LM_TILE + 1]  decay^n
  const float* dec;   // [H][2]  decay as float + float remainder
  const float* cos_t; // [positions][rd/2]
  const float* sin_t;
  int H, dk, dv, rd;
  float kscale;
  float eps;
  bool silu;          // of q, k and v as they are read
  bool raw;           // out takes S^T q as it is, without norm and gate
};
// cs [n_tiles][H][dv][dk] scratch; seqs int4 {first tile, tiles, pos0, slot}
void lm_ret_prefill(const RetArgs& a, const int4* tiles, int n_tiles,
                    const int4* seqs, int n_seqs, float* cs, bool f32,
                    hipStream_t stream);
void lm_ret_decode(const RetArgs& a, const int* pos, const int* slot, int R,
                   bool f32, hipStream_t stream);

// ---- gla.hip: a decay per key channel and token
struct GlaArgs {
  const void* q;      // rows of stride ld: q, k [H][dk], v, gate [H][dv], u
  const void* k;
  const void* v;
  const void* gate;
  const void* u;      // [rank]
  long ld;
  const void* a2;     // [H * dk][rank], [H * dk]: what makes the decay of u
  const void* a2b;
  const void* norm;   // [dv]
  float* state;       // [slots][H][dv][dk]
  void* out;          // rows of stride ldo, [H][dv]
  long ldo;
  int H, dk, dv, rank;
  float qscale, inv_tau, out_scale, eps;
};
// floats of scratch that a prompt of n_tiles tiles needs
long lm_gla_scratch(const GlaArgs& a, int n_tiles);
void lm_gla_prefill(const GlaArgs& a, const int4* tiles, int n_tiles,
                    const int4* seqs, int n_seqs, float* ws, bool f32,
                    hipStream_t stream);
void lm_gla_decode(const GlaArgs& a, const int* pos, const int* slot, int R,
                   bool f32, hipStream_t stream);

// ---- mamba2.hip / mlstm.hip: recurrences with a decay per head and token
struct GatedArgs {
  const void* q;      // rows of stride ld; head h reads group h / hpg
  const void* k;
  const void* v;      // rows of stride ld, [H][dv]
  long ld;
  int hpg;
  const void* gate;   // output gate, rows of stride ldg, [H][dv]
  const void* g0;     // mamba2: step size; mlstm: input gate   (stride ldg)
  const void* g1;     // mlstm: forget gate                     (stride ldg)
  long ldg;
  const void* b0;     // [H] biases of g0 and g1 (mamba2: b1 = A_log)
  const void* b1;
  const void* skip;   // mamba2: [H]
  const void* norm;   // mlstm: [H * dv]
  float cap;          // mlstm: of both gates
  float qscale, eps;
  float* state;       // [slots][H][dv][dk]
  float* n;           // mlstm: [slots][H][dk]
  float* m;           // mlstm: [slots][H]
  void* out;          // rows of [H * dv]
  int H, dk, dv;
};
// floats of scratch that a prompt of n_tiles tiles needs
long lm_gated_scratch(const GatedArgs& a, int n_tiles, bool mlstm);
void lm_mamba2_prefill(const GatedArgs& a, const int4* tiles, int n_tiles,
                       const int4* seqs, int n_seqs, float* cs, bool f32,
                       hipStream_t stream);
void lm_mamba2_decode(const GatedArgs& a, const int* pos, const int* slot,
                      int R, bool f32, hipStream_t stream);
void lm_mlstm_prefill(const GatedArgs& a, const int4* tiles, int n_tiles,
                      const int4* seqs, int n_seqs, float* cs, bool f32,
                      hipStream_t stream);
void lm_mlstm_decode(const GatedArgs& a, const int* pos, const int* slot,
                     int R, bool f32, hipStream_t stream);

// causal convolution over rows + silu; tail [slots][taps-1][channels]
struct ConvArgs {
  const void* in;     // rows of stride ld
  long ld;
  const void* w;      // [channels][taps]
  const void* b;      // [channels]
  float* tail;
  void* out;          // rows of [channels]
  int channels, taps;
};
void lm_causal_conv(const ConvArgs& a, const int* pos, const int* slot,
                    int n_dec, const int4* tiles, int n_tiles, const int4* seqs,
                    int n_seqs, bool f32, hipStream_t stream);

// ---- latent.hip
struct LatentArgs {
  const void* a;      // rows [q latent | kv latent | key part | head gates]
  long lda;
  int q_rank, rank, rot, rd;   // rd: rotated dimensions of the key part
  void* kc;           // [pages][64][row]: latent, key part, each padded to 8
  int row;
  const int* table;
  int max_pages;
  const float* cos_t; // [positions][rd / 2] or null
  const float* sin_t;
  int H, dim, vdim;
  int size;           // sliding window; 0: every earlier token
  float scale, eps;
};
// rows [0, T): normed query latents into cq, latent and key part into the
// cache.  keys int4 {row or -1, slot, position, 0}: the same of these tokens
// gathered into c [R][rank] and kr [R][rot].
void lm_latent_prep(const LatentArgs& a, const int* pos, const int* slot,
                    int T, const void* qw, const void* kw, void* cq,
                    const int4* keys, int R, void* c, void* kr, bool f32,
                    hipStream_t stream);
// prompt rows: blocks int4 {first row, rows <= 128, its position, place of
// position 0 among the keys}; q [T][H*(dim+rot)], k [R][H*dim], v [R][H*vdim]
void lm_latent_prefill(const LatentArgs& a, const void* q, const void* k,
                       const void* v, const void* kr, const int4* blocks,
                       int n_blocks, void* out, bool f32, hipStream_t stream);
// decode rows [0, R): qa [R][H][row] float scratch, ws R*H*nsplit*(rank+2)
bool lm_latent_decode_fits(const LatentArgs& a);
void lm_latent_decode(const LatentArgs& a, const void* q, const void* wuk,
                      const void* wuv, const int* pos, const int* slot, int R,
                      int nsplit, float* qa, float* ws, void* out, bool f32,
                      hipStream_t stream);

// ---- moe.hip: routed feed-forward
// An entry is a (token, place) pair: places 0..top-1 are the token's chosen
// experts, place `top` its shared expert (if there is one).  Entries are
// listed expert by expert (the shared one is expert E); a tile is up to
// `rows` consecutive entries of one expert.
constexpr int LM_MOE_EXPERTS = 512, LM_MOE_TOP = 64, LM_MOE_GROUPS = 64;
struct MoeArgs {
  int T, W, E, top, K;   // K: places a token has, top or top + 1
  int ff, ffs;           // inner widths of experts and shared expert (0: none)
  const float* z;        // router logits [T][ldz], the shared gate's after E
  int ldz;
  const int* table;      // null, or [vocab][top]: a token's experts, no router
  const long* tokens;    // [T]
  long vocab;
  int groups, keep;
  float scale;
  float* wts;            // [T][K]
  int* ids;              // [T][top]
  int* order;            // [T*K] token * K + place
  int4* tiles;           // {expert, first entry, rows (0: none), 0}
  int n_tiles, rows;     // bound on the tiles; rows of a full one
  const void* x;         // [T][W]
  const void* gu;        // [E][2 ff][W], gate rows first
  const void* down;      // [E][W][ff]
  const void* sgu;       // shared expert: [2 ffs][W], [W][ffs]
  const void* sdown;
  void* act;             // [T*K][lda]
  int lda;
  void* y;               // [T][K][W]
};
// z [T][n] = x [T][W] r [n][W]^T; bf16, W a multiple of 8
void lm_moe_logits(const void* x, const void* r, float* z, int T, int W, int n,
                   hipStream_t stream);
void lm_moe_plan(const MoeArgs& a, hipStream_t stream);
// rows of a tile for this problem
int lm_moe_rows(const MoeArgs& a, bool f32);
void lm_moe_experts(const MoeArgs& a, bool f32, hipStream_t stream);
