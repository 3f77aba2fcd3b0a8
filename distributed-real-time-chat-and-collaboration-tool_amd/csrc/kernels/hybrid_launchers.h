// Launchers of the kernels of models with mixed layer kinds (models/hybrid.py): Dynamic Tanh,
// latent attention, gated delta rule.  `f32` selects the activation type (0: bf16, 1: fp32).
// Same conventions as launchers.h.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace drtc {

// ---- norm_dyt.hip
int launch_dyt(int f32, void* out, float* h, const void* y, int ldy, const int* ids,
               const void* embed, const float* w, const float* b, float alpha, int rows, int W,
               hipStream_t st);
int launch_act_glu_f32(float* out, const float* gu, int64_t T, int I, int gu_stride, int act,
                       hipStream_t st);

// ---- latent_attention.hip
struct LatentPrepArgs {
  void* proj;             // [rows, ldp]: q heads at column 0 (stride dq), latent at off_kv
  int ldp, off_kv, H, dim, rot, rot_dims, R, LW;
  const float* norm_w;    // [R]
  float eps;
  const float* cos_sin;   // [positions, rot_dims]: cos | sin
  const int* positions;
  const int64_t* slots;   // cache row of each token, -1: not cached
  void* lat;              // [rows, LW] or null
  void* cache;            // [blocks * 32, LW] or null
  void* qa;               // [rows, H, LW] or null: rotated query parts at column R
  int rows;
};
int launch_latent_prep(int f32, const LatentPrepArgs& a, hipStream_t st);
int launch_latent_gather(void* out, const void* cache, const int64_t* slots, int rows,
                         int row_bytes, hipStream_t st);

struct LatentPrefillArgs {
  void* out;              // [rows, ldo], head h at column h * vdim
  int ldo;
  const void* q;          // [rows, ldq], head h at column h * (dim + rot)
  int ldq;
  const void* kv;         // [keys, ldkv]: head keys at h * dim, values at voff + h * vdim
  int ldkv, voff;
  const void* lat;        // [keys, LW]: the shared rotated key part at column R
  int LW, R, H, dim, rot, vdim;
  const int* q_cu;        // [n + 1] query rows of each sequence's portion
  const int* k_cu;        // [n + 1] key rows
  const int* ctx;         // [n] keys ahead of the portion's first query
  const int* tile_seq;
  const int* tile_q0;
  int ntiles, qtile, nseq, nq, window;   // window 0: no limit
  float scale;
  const float* sink;      // [H] or null
};
int launch_latent_prefill(int f32, const LatentPrefillArgs& a, hipStream_t st);

struct LatentDecodeArgs {
  void* out;              // [B, H, R]
  float* part_o;          // [B, H, nsplits, R]
  float* part_ml;         // [B, H, nsplits, 2]
  const void* qa;         // [B, H, LW]
  const void* cache;
  const int* block_tables;
  int bt_stride;
  const int* context_lens;
  int B, H, R, LW, window, tiles_per_split, nsplits;
  float scale;
  const float* sink;
};
int launch_latent_decode(int f32, const LatentDecodeArgs& a, hipStream_t st);
int launch_head_gemm(int f32, void* y, const void* x, const void* w, int B, int H, int N, int K,
                     int64_t yb, int64_t yh, int64_t xb, int64_t xh, hipStream_t st);
int configure_latent();

// ---- delta_rule.hip
struct DeltaArgs {
  const void* proj;       // [rows, ldp]: q | k | v channels at column 0, beta input at off_b
  int ldp, off_b;
  const void* conv;       // [rows, C] convolved + activated channels (prefill)
  const float* conv_w;    // [taps, C]
  void* ring;             // [slots, taps, C] last convolution inputs, entry = position % taps
  float* state;           // [slots, H, dim, vdim]
  const void* decay;      // [rows, H * dim] (row stride ld_decay)
  int ld_decay;
  const void* gate;       // [rows, H * vdim] (row stride ld_gate)
  int ld_gate;
  const float* a_exp;     // [H] exp(A_log)
  const float* dt_bias;   // [H * dim]
  const float* norm_w;    // [vdim]
  float eps;
  int H, Hk, dim, vdim, taps, C;
  void* out;              // [rows, H * vdim]
  // prefill: one entry per portion
  const int* seg_row;
  const int* seg_len;
  const int* seg_pos;
  const int* seg_state;
  int nseg;
  // decode: one entry per row
  const int* positions;
  const int* row_state;
  int rows;
};
int launch_short_conv(int f32, void* out, const void* proj, int ldp, const float* w,
                      const void* ring, const int* positions, const int* row_off,
                      const int* row_state, int rows, int C, int taps, hipStream_t st);
int launch_delta_scan(int f32, const DeltaArgs& a, int cpl, hipStream_t st);
int launch_delta_decode(int f32, const DeltaArgs& a, hipStream_t st);

}  // namespace drtc
