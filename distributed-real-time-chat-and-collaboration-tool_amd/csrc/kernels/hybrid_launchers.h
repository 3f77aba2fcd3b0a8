// Launchers of the kernels of models with mixed layer kinds (models/hybrid.py): Dynamic Tanh,
// latent attention, gated delta rule; convolved layer norms, talking-heads attention, gated
// average; norms in groups, grouped attention; matrix memories, the stream of joint layers.  `f32`
// selects the activation type (0: bf16, 1: fp32).  Same conventions as launchers.h.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace drtc {

// ---- norm_dyt.hip
int launch_dyt(int f32, void* out, float* h, const void* y, int ldy, const int* ids,
               const void* embed, const float* w, const float* b, float alpha, int rows, int W,
               hipStream_t st);
int launch_act_glu_f32(float* out, const float* gu, int64_t T, int I, int gu_stride, int act,
                       float limit, hipStream_t st);

// ---- latent_attention.hip
struct LatentPrepArgs {
  void* proj;             // [rows, ldp]: q heads at column 0 (stride dq), latent at off_kv (-1: queries only)
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
  const void* gate;       // [rows, ldg] gate inputs per head, or null
  int ldg;
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
  const void* gate;       // [B, ldg] gate inputs per head, or null
  int ldg;
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

// ---- norm_conv.hip
struct NormConvArgs {
  void* out[2];           // [rows, W]; the second null: one norm
  float* h_out;           // [rows, W] the residual stream after the add, or null
  const float* h_in;      // [rows, W]
  const void* y;          // [rows, ldy] added to it, or null
  int ldy;
  const int* ids;         // [rows]: the stream starts from embed rows instead
  const void* embed;
  const double* turns;    // [(W + 1) / 2] turns per position of the sinusoids, or null
  const void* w[2];       // [W] norm weights and biases (activation type)
  const void* b[2];
  const void* conv[2];    // [taps, W], or null: no convolution
  void* ring;             // [slots, norms, taps - 1, W] last normed rows
  // tiles of up to `per` tokens of a portion; tile_seg null: one row each, at positions / seg_state
  const int* tile_seg;
  const int* tile_off;
  const int* seg_row;
  const int* seg_len;
  const int* seg_pos;
  const int* seg_state;
  const int* positions;
  int ntiles, per, W, taps;
  float eps;
};
int launch_norm_conv(int f32, const NormConvArgs& a, hipStream_t st);
int launch_relu2(int f32, void* out, int64_t ldo, const void* x, int64_t rows, int cols,
                 hipStream_t st);
int launch_softcap(int f32, void* x, int64_t n, float cap, hipStream_t st);

// ---- gated_average.hip
struct GatedAverageArgs {
  const void* proj;       // [rows, ldp]: z' at column 0, x' at off_x, g' at off_g
  int ldp, off_x, off_g;
  const float* zb;        // [C]
  const float* xb;
  float* state;           // [slots, C]
  void* out;              // [rows, ldo]
  int ldo, C;
  const int* seg_row;     // prefill: one entry per portion
  const int* seg_len;
  const int* seg_pos;
  const int* seg_state;
  int nseg;
  // long portions: chunks of `chunk` tokens, a portion's one after the other (nchunks 0: none)
  const int* chunk_seg;
  const int* chunk_off;
  float* maps;            // [nchunks, 2, C]
  int nchunks, chunk;
  const int* positions;   // decode: one entry per row
  const int* row_state;
  int rows;
};
int launch_gated_scan(int f32, const GatedAverageArgs& a, hipStream_t st);
int launch_gated_decode(int f32, const GatedAverageArgs& a, hipStream_t st);

// ---- talking_attention.hip
struct HeadPrepArgs {
  const void* proj;       // [rows, ldp]: query heads at column 0, keys at off_k, values at off_v
  int ldp, off_k, off_v, H, G, dim, dimp, vdimp;
  const float* qb;        // biases, padded as the heads
  const float* kb;
  const float* vb;
  const float* qn;        // [dimp] norm weights
  const float* kn;
  float eps;
  const int64_t* slots;   // cache row of each token, -1: not cached
  void* q;                // [rows, H, dimp]
  void* k;                // cache
  void* v;
  int rows;
};
int launch_head_prep(int f32, const HeadPrepArgs& a, hipStream_t st);

// ---- talking_decode.hip
struct TalkDecodeArgs {
  void* out;              // [B, ldo], head h at column h * vdimp
  int ldo;
  const void* q;          // [B, H, dimp]
  const void* k;          // cache
  const void* v;
  float* plane;           // [blocks, H, 32] scores, log2 units
  float* part_ml;         // [B, nsplits, H, 2]
  float* part_o;          // [B, nsplits, H, vdimp] (nsplits > 1)
  const int* block_tables;
  int bt_stride;
  const int* context_lens;
  const float* sink;      // [H] or null
  const float* talk;      // [H, H]
  float scale;
  int B, H, G, dimp, vdimp, per, nsplits;  // per: cache blocks of a split
};
int launch_talk_decode(int f32, const TalkDecodeArgs& a, hipStream_t st);

// ---- talking_attention.hip
struct TalkPrefillArgs {
  void* out;              // [nq, ldo]
  int ldo;
  const void* q;          // [nq, H, dimp]
  const void* k;          // cache
  const void* v;
  float* stats;           // [nq, H] (MFMA form)
  const int* q_cu;        // [nseq + 1] query rows of each portion
  const int* start;       // [nseq] position of its first query
  const int* block_tables;
  int bt_stride;
  const int* tile_seq;    // 16-query tiles of the mixing sweep
  const int* tile_q0;
  const int* stile_seq;   // 64-query tiles of the denominators' sweep
  const int* stile_q0;
  int ntiles, nstiles, nseq, nq;
  const float* sink;
  const float* talk;
  float scale;
  int H, G, dimp, vdimp, mfma;
};
int launch_talk_prefill(int f32, const TalkPrefillArgs& a, hipStream_t st);
int configure_talking();

// ---- norm_group.hip
struct GroupRmsArgs {
  void* out;              // [rows, ldo], columns beyond W zero
  int ldo;
  float* h;               // [rows, W] the residual stream, updated
  const void* y;          // [rows, ldy] added to it times s, or null
  int ldy;
  const float* s;         // [W]
  const int* ids;         // [rows]: the stream starts from embed rows times embed_scale instead
  const void* embed;
  float embed_scale;
  const float* w;         // [W]
  int W, groups;
  float eps;
  int rows;
};
int launch_group_rms(int f32, const GroupRmsArgs& a, hipStream_t st);

// ---- grouped_attention.hip
struct AttnPrepArgs {
  const void* proj;       // [rows, ldp]: query heads at column 0, keys at off_k, values at off_v
  int ldp, off_k, off_v, H, G, dimp, vdimp;
  const float* conv;      // [taps, C], C = (H + G) dimp + G vdimp channels q | k | v
  int taps;
  void* ring;             // [slots, taps - 1, C] last projected rows, entry = position % (taps - 1)
  const float* cos_sin;   // [positions, rot_dims]: cos | sin
  int rot_dims;
  const int64_t* slots;   // cache row of each token, -1: not cached
  void* q;                // [rows, H, dimp]
  void* k;                // cache
  void* v;
  void* v_first;          // [rows, G vdim] or null: this layer's values go there, or (mix) are
  int mix;                // mixed with what it holds
  int vdim;
  float lam;
  // tiles of up to `per` tokens of a portion; tile_seg null: one row each, at positions / row_state
  const int* tile_seg;
  const int* tile_off;
  const int* seg_row;
  const int* seg_len;
  const int* seg_pos;
  const int* seg_state;
  const int* positions;
  const int* row_state;
  int ntiles, per;
};
int launch_attn_prep(int f32, const AttnPrepArgs& a, hipStream_t st);

struct GroupedAttnArgs {
  void* out;              // [rows, ldo], head h at column h * vdimp
  int ldo;
  const void* q;          // [rows, H, dimp]
  const void* k;          // cache
  const void* v;
  const void* gate;       // [rows, ldg] gate inputs per head, or null
  int ldg;
  const int* block_tables;  // of each portion / decode row
  int bt_stride, H, G, dimp, vdimp, sink;
  float scale, cap;       // cap 0: scores as they are
  // prompt portions
  const int* q_cu;        // [nseq + 1] query rows; null: decode
  const int* start;       // [nseq] position of the first query
  const int* tile_seq;    // tiles of qtile (query, head) rows of one kv head
  const int* tile_row;
  int ntiles, qtile, nseq;
  // decode
  const int* context_lens;
  float* part_ml;         // [B, nsplits, H, 2]
  float* part_o;          // [B, nsplits, H, vdimp]
  int B, per, nsplits;    // per: cache blocks of a split
};
int launch_grouped_any(int f32, const GroupedAttnArgs& a, int rows, hipStream_t st);
int launch_grouped_prefill(const GroupedAttnArgs& a, hipStream_t st);
int configure_grouped();

// ---- grouped_decode.hip
int launch_grouped_decode(const GroupedAttnArgs& a, hipStream_t st);
int configure_grouped_decode();

// ---- memory_scan.hip
struct MemoryArgs {
  const void* proj;       // [rows, ldp]: query heads at column 0, keys, values, read-out gates and
  int ldp, off_k, off_v, off_g, off_i, off_f;  // (log_decay null) input and forget gates behind
  int H, dim, vdim;
  float q_scale, k_scale;  // on queries, on keys (after the rotation)
  const float* cos_sin;   // [positions, rot_dims]: cos | sin
  int rot_dims;
  const float* log_decay;  // [H], or null: gates
  const float* i_bias;    // [H]
  const float* f_bias;
  float cap;
  const float* norm_w;    // [H * vdim] or null
  int silu;               // read-out gate: 1 silu, 0 sigmoid
  float eps;
  float* state;           // [slots, H, dim, vdim]
  float* nrm;             // [slots, H, dim] (gates)
  float* top;             // [slots, H, slices] running maximum (gates)
  int slices;             // a head's columns are split over this many workgroups
  void* out;              // [rows, ldo], head h at column h * vdim
  int ldo;
  const int* seg_row;     // prefill: one entry per portion
  const int* seg_len;
  const int* seg_pos;
  const int* seg_state;
  int nseg;
  const int* positions;   // decode: one entry per row
  const int* row_state;
  int rows;
};
int launch_memory_scan(int f32, const MemoryArgs& a, int plain, hipStream_t st);
int launch_memory_decode(int f32, const MemoryArgs& a, hipStream_t st);
int configure_memory();

// ---- norm_side.hip
struct SideNormArgs {
  void* out;              // [rows, ldo], columns beyond W zero
  int ldo;
  float* h;               // [rows, W] the residual stream, updated
  const void* y;          // [rows, ldy] RMS-normed, times yw, added to it; or null
  int ldy;
  const float* yw;        // [W]
  const int* ids;         // [rows]: the stream starts from embed rows times embed_scale instead
  const void* embed;
  float embed_scale;
  const float* w;         // [W]
  int W;
  float eps;
  int rows;
};
int launch_side_norm(int f32, const SideNormArgs& a, hipStream_t st);
int launch_stream_add(int f32, void* out, float* h, const void* y, int64_t ldy, int rows, int W,
                      hipStream_t st);
int launch_side_gate_gemm(void* out, const void* x, const void* w, const void* embed, int64_t lde,
                          int off, const int* ids, int T, int N, int K, hipStream_t st);
int launch_side_gate(int f32, void* out, const void* z, const void* embed, int64_t lde, int off,
                     const int* ids, int rows, int dim, hipStream_t st);

}  // namespace drtc
