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
void lm_embed_norm(const long* tokens, const void* embed, float* x,
                   const void* w, const void* b, void* h, int T, int W,
                   long vocab, float eps, bool f32, hipStream_t stream);
void lm_residual_norm(float* x, const void* y, const void* pw, const void* pb,
                      float mult, const void* nw, const void* nb, void* h,
                      const int* rows, int T, int W, float eps, bool store_x,
                      bool f32, hipStream_t stream);
void lm_gelu_erf(const void* in, void* out, long n, bool f32,
                 hipStream_t stream);

// ---- attn.hip / attn_decode.hip
struct AttnArgs {
  void* qkv;          // rows of [heads*dim | kv_heads*dim | kv_heads*vdim]
  long ld;            // row stride of qkv (elements)
  void* kc;
  void* vc;
  void* out;          // rows of [heads*vdim]
  const void* qw;     // per-head RMS weights or null
  const void* kw;
  const void* sink;   // [heads] or null
  const int* table;
  int max_pages;
  int H, G, dim, vdim;
  int size;           // chunk length in tokens; 0 = plain causal
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
};
// cs [n_tiles][H][dv][dk] scratch; seqs int4 {first tile, tiles, pos0, slot}
void lm_ret_prefill(const RetArgs& a, const int4* tiles, int n_tiles,
                    const int4* seqs, int n_seqs, float* cs, bool f32,
                    hipStream_t stream);
void lm_ret_decode(const RetArgs& a, const int* pos, const int* slot, int R,
                   bool f32, hipStream_t stream);
