// Gated delta rule with per-channel decay (gfx950): short causal convolutions, the recurrence,
// and the gated output norm.
//
// Per head, with the 32-bit state S [dim, vdim] of a sequence:
//   S <- g * S (rows),  u = beta (v - S^T k),  S <- S + k u^T,  o = S^T q
//   out = o / rms(o) * w * sigmoid(gate)
// The columns of S are independent, so a column lives in the registers of 8 lanes: lane 8 c + p
// of a wave holds rows {32 m + 4 p .. + 3} of CPL columns, both products with the decayed state
// are taken in one pass (S^T q = (gS)^T q + u (k.q)) and reduced with three DPP adds.  CPL
// columns share each LDS read of k, q, g.
//   short_conv_kernel    prompt portions: convolution + SiLU of the packed rows; inputs ahead
//                        of a portion come from the sequence's ring of the last `taps` inputs
//   delta_chunk_kernel   one workgroup per (portion, head): 8 tokens at a time in matrix form on
//                        the fp32 MFMA (derivation at the kernel)
//   delta_scan_kernel    the same token by token, for sizes the chunk form does not take
//   delta_decode_kernel  one workgroup per (sequence, head): all of it for one token; the
//                        state streams through registers once
// A ring entry is position % taps: the entry a token writes is the one its own convolution no
// longer reads, so heads sharing a key never race on it.
#include "hybrid_launchers.h"
#include "typed.h"

#include <algorithm>

namespace drtc {

DRTC_DEVICE float silu_f(float x) { return x / (1.f + expf(-x)); }
// result rounded to bf16: hardware exp and reciprocal
template <class T>
DRTC_DEVICE float silu_as(float x) { return silu_f(x); }
template <>
DRTC_DEVICE float silu_as<bf16_t>(float x) {
  return x * __builtin_amdgcn_rcpf(1.f + fast_exp2(-kLog2e * x));
}
DRTC_DEVICE float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
DRTC_DEVICE float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// ------------------------------------------------------------------ convolution
// VEC channels per thread, 16 consecutive rows per workgroup (the rows behind a row stay in
// the L1).  TAPS 0: any number of taps.
constexpr int kConvRows = 16;

template <class T, int VEC, int TAPS>
__global__ __launch_bounds__(256) void short_conv_kernel(
    T* __restrict__ out, const T* __restrict__ proj, int ldp, const float* __restrict__ w,
    const T* __restrict__ ring, const int* __restrict__ positions,
    const int* __restrict__ row_off, const int* __restrict__ row_state, int rows, int C,
    int taps_rt) {
  const int taps = TAPS ? TAPS : taps_rt;
  const int c = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (c >= C) return;
  float wr[TAPS ? TAPS : 1][VEC];
  auto loadw = [&](float (&d)[VEC], int j) {
#pragma unroll
    for (int i = 0; i < VEC; ++i) d[i] = w[(int64_t)j * C + c + i];
  };
  if constexpr (TAPS != 0) {
#pragma unroll
    for (int j = 0; j < TAPS; ++j) loadw(wr[j], j);
  }
  auto loadx = [&](float (&d)[VEC], const T* p) {
    if constexpr (VEC == 8) load8(d, p);
    else d[0] = to_f32(*p);
  };
  const int r1 = min(rows, (int)(blockIdx.x + 1) * kConvRows);
  // the inputs of the rows behind: hist[j] belongs to row - 1 - j while ``have`` > j
  float hist[TAPS > 1 ? TAPS - 1 : 1][VEC];
  int have = 0;
  for (int row = blockIdx.x * kConvRows; row < r1; ++row) {
    const int slot = row_state[row];
    float acc[VEC], x0[VEC];
#pragma unroll
    for (int i = 0; i < VEC; ++i) acc[i] = 0.f;
    if (slot >= 0) {
      const int off = row_off[row], pos = positions[row];
      loadx(x0, proj + (int64_t)row * ldp + c);
      auto add = [&](const float (&x)[VEC], const float (&wj)[VEC]) {
#pragma unroll
        for (int i = 0; i < VEC; ++i) acc[i] += x[i] * wj[i];
      };
      auto fetch = [&](float (&x)[VEC], int j) {  // j tokens back; false: before the start
        if (j <= off) loadx(x, proj + (int64_t)(row - j) * ldp + c);
        else if (j <= pos) loadx(x, ring + ((int64_t)slot * taps + (pos - j) % taps) * C + c);
        else return false;
        return true;
      };
      if constexpr (TAPS != 0) {
        add(x0, wr[TAPS - 1]);
#pragma unroll
        for (int j = 1; j < TAPS; ++j) {
          if (j <= have && j <= off) add(hist[j - 1], wr[TAPS - 1 - j]);
          else {
            float x[VEC];
            if (fetch(x, j)) add(x, wr[TAPS - 1 - j]);
          }
        }
      } else {
        loadw(wr[0], taps - 1);
        add(x0, wr[0]);
        for (int j = 1; j < taps; ++j) {
          float x[VEC];
          loadw(wr[0], taps - 1 - j);
          if (fetch(x, j)) add(x, wr[0]);
        }
      }
#pragma unroll
      for (int i = 0; i < VEC; ++i) acc[i] = silu_as<T>(acc[i]);
      if constexpr (TAPS > 1) {
#pragma unroll
        for (int j = TAPS - 2; j > 0; --j)
#pragma unroll
          for (int i = 0; i < VEC; ++i) hist[j][i] = hist[j - 1][i];
#pragma unroll
        for (int i = 0; i < VEC; ++i) hist[0][i] = x0[i];
        ++have;
      }
    } else {
      have = 0;
    }
    T* op = out + (int64_t)row * C + c;
    if constexpr (VEC == 8) store8(op, acc);
    else *op = from_f32<T>(acc[0]);
  }
}

template <class T>
static void conv_t(void* out, const void* proj, int ldp, const float* w, const void* ring,
                   const int* positions, const int* row_off, const int* row_state, int rows,
                   int C, int taps, hipStream_t st) {
  const bool vec = C % 8 == 0 && ldp % 8 == 0;
  const int per = 256 * (vec ? 8 : 1);
  const dim3 grid((rows + kConvRows - 1) / kConvRows, (C + per - 1) / per);
#define DRTC_CONV(V, N)                                                                       \
  short_conv_kernel<T, V, N><<<grid, dim3(256), 0, st>>>((T*)out, (const T*)proj, ldp, w,     \
                                                         (const T*)ring, positions, row_off,  \
                                                         row_state, rows, C, taps)
  if (vec && taps == 4) DRTC_CONV(8, 4);
  else if (vec) DRTC_CONV(8, 0);
  else DRTC_CONV(1, 0);
#undef DRTC_CONV
}

int launch_short_conv(int f32, void* out, const void* proj, int ldp, const float* w,
                      const void* ring, const int* positions, const int* row_off,
                      const int* row_state, int rows, int C, int taps, hipStream_t st) {
  if (rows == 0) return 0;
  if (taps < 1) return -1;
  if (f32) conv_t<float>(out, proj, ldp, w, ring, positions, row_off, row_state, rows, C, taps, st);
  else conv_t<bf16_t>(out, proj, ldp, w, ring, positions, row_off, row_state, rows, C, taps, st);
  return (int)hipGetLastError();
}

// ------------------------------------------------------------------ the recurrence
// This lane's rows of CPL consecutive columns, from / to S [dim, vdim].
template <int DPL, int CPL>
struct StateTile {
  float s[DPL][CPL];
  DRTC_DEVICE void zero() {
#pragma unroll
    for (int i = 0; i < DPL; ++i)
#pragma unroll
      for (int c = 0; c < CPL; ++c) s[i][c] = 0.f;
  }
  DRTC_DEVICE static int row_of(int i, int p) { return 32 * (i >> 2) + 4 * p + (i & 3); }
  DRTC_DEVICE void load(const float* S, int col, int p, int dim, int vdim) {
    if constexpr (CPL % 4 == 0) {
      if ((vdim & 3) == 0) {
#pragma unroll
        for (int i = 0; i < DPL; ++i) {
          const int r = row_of(i, p);
#pragma unroll
          for (int c = 0; c < CPL; c += 4) {
            f32x4 v = {0.f, 0.f, 0.f, 0.f};
            if (r < dim && col + c < vdim)
              v = *reinterpret_cast<const f32x4*>(S + (int64_t)r * vdim + col + c);
#pragma unroll
            for (int j = 0; j < 4; ++j) s[i][c + j] = v[j];
          }
        }
        return;
      }
    }
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int r = row_of(i, p);
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        s[i][c] = r < dim && col + c < vdim ? S[(int64_t)r * vdim + col + c] : 0.f;
    }
  }
  DRTC_DEVICE void store(float* S, int col, int p, int dim, int vdim) const {
    if constexpr (CPL % 4 == 0) {
      if ((vdim & 3) == 0) {
#pragma unroll
        for (int i = 0; i < DPL; ++i) {
          const int r = row_of(i, p);
#pragma unroll
          for (int c = 0; c < CPL; c += 4) {
            f32x4 v;
#pragma unroll
            for (int j = 0; j < 4; ++j) v[j] = s[i][c + j];
            if (r < dim && col + c < vdim)
              *reinterpret_cast<f32x4*>(S + (int64_t)r * vdim + col + c) = v;
          }
        }
        return;
      }
    }
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int r = row_of(i, p);
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        if (r < dim && col + c < vdim) S[(int64_t)r * vdim + col + c] = s[i][c];
    }
  }
  // One token: k, q, g rows in LDS (padded to 8 DPL), qk = k.q; o[c] = the read-out.
  DRTC_DEVICE void token(const float* k, const float* q, const float* g, int p, float beta,
                         float qk, const float (&v)[CPL], float (&o)[CPL]) {
    float kk[DPL], ks[CPL], qs[CPL];
#pragma unroll
    for (int c = 0; c < CPL; ++c) ks[c] = qs[c] = 0.f;
#pragma unroll
    for (int m = 0; m < DPL / 4; ++m) {
      const int at = 32 * m + 4 * p;
      const f32x4 k4 = *reinterpret_cast<const f32x4*>(k + at);
      const f32x4 q4 = *reinterpret_cast<const f32x4*>(q + at);
      const f32x4 g4 = *reinterpret_cast<const f32x4*>(g + at);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        kk[4 * m + j] = k4[j];
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
          const float x = s[4 * m + j][c] * g4[j];
          s[4 * m + j][c] = x;
          ks[c] += k4[j] * x;
          qs[c] += q4[j] * x;
        }
      }
    }
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const float u = beta * (v[c] - sum8(ks[c]));
      o[c] = sum8(qs[c]) + u * qk;
#pragma unroll
      for (int i = 0; i < DPL; ++i) s[i][c] += kk[i] * u;
    }
  }
};

// Convolution inputs of a portion's last `taps` tokens into the ring, by the workgroup of head h
// (its values; the group's first head also its queries and keys).
template <class T>
DRTC_DEVICE void keep_ring(const DeltaArgs& a, int slot, int h, int n, int row0, int pos0) {
  const int grp = a.H / a.Hk, hk = h / grp;
  const int cq = hk * a.dim, ck = (a.Hk + hk) * a.dim, cv = 2 * a.Hk * a.dim + h * a.vdim;
  const T* proj = (const T*)a.proj;
  T* ring = (T*)a.ring + (int64_t)slot * a.taps * a.C;
  const int nr = min(n, a.taps), own = h % grp == 0 ? 2 * a.dim : 0;
  for (int k = threadIdx.x; k < nr * (own + a.vdim); k += blockDim.x) {
    const int j = k / (own + a.vdim), i = k % (own + a.vdim);
    const int c = i < own ? (i < a.dim ? cq + i : ck + i - a.dim) : cv + i - own;
    const int t = n - nr + j;
    ring[(int64_t)((pos0 + t) % a.taps) * a.C + c] = proj[(int64_t)(row0 + t) * a.ldp + c];
  }
}

template <int DPL>
struct ScanShape {
  static constexpr int DP = 8 * DPL;             // padded key size
  static constexpr int CT = DPL <= 16 ? 16 : 8;  // tokens staged at a time
};

template <class T, int DPL, int CPL>
__global__ __launch_bounds__(512) void delta_scan_kernel(DeltaArgs a) {
  constexpr int DP = ScanShape<DPL>::DP, CT = ScanShape<DPL>::CT;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int seg = blockIdx.x, h = blockIdx.y;
  const int slot = a.seg_state[seg];
  const int n = a.seg_len[seg], row0 = a.seg_row[seg], pos0 = a.seg_pos[seg];
  const int tid = threadIdx.x, nthr = blockDim.x;
  T* out = (T*)a.out;
  const int ldo = a.H * a.vdim;
  if (slot < 0) {  // padding row of a decode bucket
    for (int i = tid; i < n * a.vdim; i += nthr)
      out[(int64_t)(row0 + i / a.vdim) * ldo + h * a.vdim + i % a.vdim] = from_f32<T>(0.f);
    return;
  }
  const int dvp = (a.vdim + 3) & ~3;
  float* ks = sm;
  float* qs = ks + CT * DP;
  float* gs = qs + CT * DP;
  float* vs = gs + CT * DP;
  float* os = vs + CT * dvp;
  float* qk = os + CT * dvp;
  float* bs = qk + CT;

  const int lane = tid & 63, p = lane & 7;
  const int col = ((tid >> 6) * 8 + (lane >> 3)) * CPL;
  const int grp = a.H / a.Hk, hk = h / grp;
  const int cq = hk * a.dim, ck = (a.Hk + hk) * a.dim, cv = 2 * a.Hk * a.dim + h * a.vdim;
  const float aexp = a.a_exp[h], qscale = rsqrtf((float)a.dim);
  float* S = a.state + ((int64_t)slot * a.H + h) * a.dim * a.vdim;
  StateTile<DPL, CPL> st;
  if (pos0 > 0) st.load(S, col, p, a.dim, a.vdim);
  else st.zero();
  const int l16 = tid & 15, g16 = tid >> 4, n16 = nthr >> 4;
  const T* conv = (const T*)a.conv;
  const T* proj = (const T*)a.proj;
  const T* dec = (const T*)a.decay;
  const T* gate = (const T*)a.gate;

  for (int t0 = 0; t0 < n; t0 += CT) {
    const int nt = min(CT, n - t0);
    for (int t = g16; t < nt; t += n16) {  // 16 lanes per token
      const int64_t row = row0 + t0 + t;
      const T* cr = conv + row * a.C;
      float sq = 0.f, sk = 0.f, dot = 0.f;
      for (int i = l16; i < DP; i += 16) {
        const float q = i < a.dim ? to_f32(cr[cq + i]) : 0.f;
        const float k = i < a.dim ? to_f32(cr[ck + i]) : 0.f;
        sq += q * q;
        sk += k * k;
        dot += q * k;
        gs[t * DP + i] = i < a.dim
            ? expf(-aexp * softplus_f(to_f32(dec[row * a.ld_decay + h * a.dim + i]) +
                                      a.dt_bias[h * a.dim + i]))
            : 1.f;
        qs[t * DP + i] = q;
        ks[t * DP + i] = k;
      }
      const float rq = qscale / sqrtf(sum16(sq) + 1e-6f), rk = 1.f / sqrtf(sum16(sk) + 1e-6f);
      dot = sum16(dot);
      for (int i = l16; i < DP; i += 16) {
        qs[t * DP + i] *= rq;
        ks[t * DP + i] *= rk;
      }
      for (int i = l16; i < a.vdim; i += 16) vs[t * dvp + i] = to_f32(cr[cv + i]);
      if (l16 == 0) {
        qk[t] = dot * rq * rk;
        bs[t] = sigmoid_f(to_f32(proj[row * a.ldp + a.off_b + h]));
      }
    }
    __syncthreads();
    if (col < a.vdim) {
      for (int t = 0; t < nt; ++t) {
        float v[CPL], o[CPL];
#pragma unroll
        for (int c = 0; c < CPL; ++c) v[c] = col + c < a.vdim ? vs[t * dvp + col + c] : 0.f;
        st.token(ks + t * DP, qs + t * DP, gs + t * DP, p, bs[t], qk[t], v, o);
        if (p == 0) {
#pragma unroll
          for (int c = 0; c < CPL; ++c)
            if (col + c < a.vdim) os[t * dvp + col + c] = o[c];
        }
      }
    }
    __syncthreads();
    for (int t = g16; t < nt; t += n16) {
      const int64_t row = row0 + t0 + t;
      float so = 0.f;
      for (int i = l16; i < a.vdim; i += 16) {
        const float o = os[t * dvp + i];
        so += o * o;
      }
      const float r = 1.f / sqrtf(sum16(so) / (float)a.vdim + a.eps);
      for (int i = l16; i < a.vdim; i += 16)
        out[row * ldo + h * a.vdim + i] =
            from_f32<T>(os[t * dvp + i] * r * a.norm_w[i] *
                        sigmoid_f(to_f32(gate[row * a.ld_gate + h * a.vdim + i])));
    }
    // the next chunk's staging writes ks / qs / gs / vs, last read before the barrier above;
    // os is written again only after the next barrier
  }
  if (col < a.vdim) st.store(S, col, p, a.dim, a.vdim);
  keep_ring<T>(a, slot, h, n, row0, pos0);
}


// ------------------------------------------------------------------ chunks on the fp32 MFMA
// For the tokens 1..8 of a chunk let c_i be the running sum of log2 g (per key channel),
// S the state ahead of the chunk, E_i = 2^{c_i}.  Unrolling the recurrence,
//   S_i = E_i * S + sum_{j <= i} (2^{c_i - c_j} * k_j) u_j^T
//   u_i = beta_i (v_i - (E_i * k_i)^T S - sum_{j < i} A_ij u_j),  A_ij = k_i . (2^{c_i - c_j} * k_j)
//   o_i = (E_i * q_i)^T S + sum_{j <= i} B_ij u_j,                B_ij = q_i . (2^{c_i - c_j} * k_j)
// (exponents of differences are never positive: no decay is divided by).  With R = V - (E*K)^T S,
//   U = (I + diag(beta) A)^{-1} diag(beta) R = M_U R,   O = (E*Q)^T S + B U = (E*Q)^T S + M_O R.
// All products with S are 16-row MFMAs - 8 key rows and 8 query rows of a chunk - and so are
// the products with [M_U; M_O]; the 8 x 8 inverse is a forward substitution shared by all
// columns.  A wave keeps 32 columns of S as accumulator tiles: their layout (row 4 g + r of
// lane group g) is also a B operand with k-step r taking dim 4 g + r, so S feeds its own
// products without lane movement.
// 16 tokens (two chunks) are staged at a time; their global loads are in flight while the
// previous 16 are computed.
DRTC_DEVICE f32x4 mfma_f32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
DRTC_DEVICE float log2_fast(float x) { return __builtin_amdgcn_logf(x); }
// softplus by hardware exp2 / log2; for large -x its series, where 1 + e^x would round
DRTC_DEVICE float softplus_hw(float x) {
  const float e = fast_exp2(x * kLog2e);
  const float l = log2_fast(1.f + e) * (1.f / kLog2e);
  return x > 20.f ? x : x < -6.f ? e * (1.f - e * (0.5f - e * (1.f / 3.f))) : l;
}
DRTC_DEVICE float sigmoid_hw(float x) {
  return 1.f / (1.f + fast_exp2(-kLog2e * x));
}

template <int DT, int NTHR>
struct ChunkLds {
  static constexpr int DP = 16 * DT, DS = DP + 4, KD = DP + 16;
  static constexpr int NW = NTHR / 64, VS = 32 * NW + 4, UB = 36;
  static constexpr int k = 0, q = k + 16 * DS, c = q + 16 * DS, kd = c + 16 * DS;
  static constexpr int gt = kd + 16 * KD, v = gt + 2 * DP, mm = v + 16 * VS, beta = mm + 256;
  static constexpr int tmp = beta + 16;  // pair sums [2][2][2][64], then each wave's U [8][UB]
  static constexpr int tmp_n = NW * 8 * UB > 512 ? NW * 8 * UB : 512;
  static constexpr size_t BYTES = sizeof(float) * (size_t)(tmp + tmp_n);
};

template <class T, int DT, int NTHR>
__global__ __launch_bounds__(NTHR, 2) void delta_chunk_kernel(DeltaArgs a) {
  using L = ChunkLds<DT, NTHR>;
  constexpr int NVV = NTHR / 256;  // 8-column vectors of v per lane of a token's 16
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int seg = blockIdx.x, h = blockIdx.y;
  const int slot = a.seg_state[seg];
  const int n = a.seg_len[seg], row0 = a.seg_row[seg], pos0 = a.seg_pos[seg];
  const int tid = threadIdx.x;
  T* out = (T*)a.out;
  const int ldo = a.H * a.vdim;
  if (slot < 0) {  // padding row of a decode bucket
    for (int i = tid; i < n * a.vdim; i += NTHR)
      out[(int64_t)(row0 + i / a.vdim) * ldo + h * a.vdim + i % a.vdim] = from_f32<T>(0.f);
    return;
  }
  const int w = wave_id_uniform(), lane = tid & 63, col = lane & 15, g = lane >> 4;
  const int grp = a.H / a.Hk, hk = h / grp;
  const int cq = hk * a.dim, ck = (a.Hk + hk) * a.dim, cv = 2 * a.Hk * a.dim + h * a.vdim;
  const float decay_scale = -a.a_exp[h] * kLog2e, qscale = rsqrtf((float)a.dim);
  float* S = a.state + ((int64_t)slot * a.H + h) * a.dim * a.vdim;
  const bool owner = 32 * w < a.vdim;  // this wave has columns

  f32x4 st[DT][2];
#pragma unroll
  for (int t = 0; t < DT; ++t)
#pragma unroll
    for (int ct = 0; ct < 2; ++ct)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * t + 4 * g + r, x = 32 * w + 16 * ct + col;
        st[t][ct][r] = pos0 > 0 && d < a.dim && x < a.vdim ? S[(int64_t)d * a.vdim + x] : 0.f;
      }

  // staging: 16 lanes per token, 8 elements each
  const int tok = tid >> 4, e8 = (tid & 15) * 8;
  const bool stager = tok < 16;
  float dtb[8], nw[NVV][8];
#pragma unroll
  for (int j = 0; j < 8; ++j) dtb[j] = e8 + j < a.dim ? a.dt_bias[h * a.dim + e8 + j] : 0.f;
#pragma unroll
  for (int i = 0; i < NVV; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int x = 128 * i + e8 + j;
      nw[i][j] = x < a.vdim ? a.norm_w[x] : 0.f;
    }
  struct alignas(16) Vec { T x[8]; };
  Vec pq, pk, pd, pv[NVV], pg[NVV], ng[NVV];
  T pb = from_f32<T>(0.f);
  auto get = [](float (&d)[8], const Vec& s) {
#pragma unroll
    for (int j = 0; j < 8; ++j) d[j] = to_f32(s.x[j]);
  };
  auto prefetch = [&](int t0) {
    if (!stager || t0 + tok >= n) return;
    const int64_t row = row0 + t0 + tok;
    const T* cr = (const T*)a.conv + row * a.C;
    if (e8 < a.dim) {
      pq = *(const Vec*)(cr + cq + e8);
      pk = *(const Vec*)(cr + ck + e8);
      pd = *(const Vec*)((const T*)a.decay + row * a.ld_decay + h * a.dim + e8);
    }
#pragma unroll
    for (int i = 0; i < NVV; ++i)
      if (128 * i + e8 < a.vdim) {
        pv[i] = *(const Vec*)(cr + cv + 128 * i + e8);
        ng[i] = *(const Vec*)((const T*)a.gate + row * a.ld_gate + h * a.vdim + 128 * i + e8);
      }
    pb = ((const T*)a.proj)[row * a.ldp + a.off_b + h];
  };
  prefetch(0);

  for (int t0 = 0; t0 < n; t0 += 16) {
    const bool live = stager && t0 + tok < n;
    if (stager) {
      float q[8], k[8], l[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) q[j] = k[j] = l[j] = 0.f;
      if (live && e8 < a.dim) {
        get(q, pq);
        get(k, pk);
        get(l, pd);
#pragma unroll
        for (int j = 0; j < 8; ++j) l[j] = decay_scale * softplus_hw(l[j] + dtb[j]);
      }
      float sq = 0.f, sk = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        sq += q[j] * q[j];
        sk += k[j] * k[j];
      }
      const float rq = qscale / sqrtf(sum16(sq) + 1e-6f), rk = 1.f / sqrtf(sum16(sk) + 1e-6f);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        q[j] *= rq;
        k[j] *= rk;
      }
      if (e8 < L::DP) {
        store8(sm + L::q + tok * L::DS + e8, q);
        store8(sm + L::k + tok * L::DS + e8, k);
        store8(sm + L::c + tok * L::DS + e8, l);
      }
#pragma unroll
      for (int i = 0; i < NVV; ++i)
        if (128 * i + e8 < L::VS - 4) {
          float v[8];
#pragma unroll
          for (int j = 0; j < 8; ++j) v[j] = 0.f;
          if (live && 128 * i + e8 < a.vdim) get(v, pv[i]);
          store8(sm + L::v + tok * L::VS + 128 * i + e8, v);
          pg[i] = ng[i];
        }
      if ((tid & 15) == 0) sm[L::beta + tok] = live ? sigmoid_hw(to_f32(pb)) : 0.f;
    }
    prefetch(t0 + 16);
    __syncthreads();
    // running decays of the two chunks; keys decayed to the chunk's end
    if (tid < 2 * L::DP) {
      const int ch = tid / L::DP, d = tid % L::DP;
      float* c = sm + L::c + 8 * ch * L::DS + d;
      float run[8], acc = 0.f;
#pragma unroll
      for (int t = 0; t < 8; ++t) run[t] = acc += c[t * L::DS];
#pragma unroll
      for (int t = 0; t < 8; ++t) {
        c[t * L::DS] = run[t];
        sm[L::kd + (8 * ch + t) * L::KD + d] =
            sm[L::k + (8 * ch + t) * L::DS + d] * fast_exp2(acc - run[t]);
      }
      sm[L::gt + ch * L::DP + d] = fast_exp2(acc);
    }
    __syncthreads();
    // A and B: one (i, j) pair per lane, two halves of the channels
    if (tid < 256) {
      const int ch = tid >> 7, half = (tid >> 6) & 1, i = (tid >> 3) & 7, j = tid & 7;
      const float* ki = sm + L::k + (8 * ch + i) * L::DS + half * (L::DP / 2);
      const float* kj = sm + L::k + (8 * ch + j) * L::DS + half * (L::DP / 2);
      const float* qi = ki + (L::q - L::k);
      const float* ci = ki + (L::c - L::k);
      const float* cj = kj + (L::c - L::k);
      float A = 0.f, B = 0.f;
#pragma unroll 2
      for (int d = 0; d < L::DP / 2; d += 4) {
        const f32x4 k4 = *(const f32x4*)(ki + d), q4 = *(const f32x4*)(qi + d);
        const f32x4 x4 = *(const f32x4*)(kj + d);
        const f32x4 c4 = *(const f32x4*)(ci + d), z4 = *(const f32x4*)(cj + d);
#pragma unroll
        for (int m = 0; m < 4; ++m) {
          const float y = x4[m] * fast_exp2(fminf(c4[m] - z4[m], 0.f));
          A += k4[m] * y;
          B += q4[m] * y;
        }
      }
      float* pr = sm + L::tmp + ch * 256 + half * 64 + i * 8 + j;
      pr[0] = A;
      pr[128] = B;
    }
    __syncthreads();
    if (w < 2) {  // [M_U; M_O] of chunk w, column lane & 7
      const float* pr = sm + L::tmp + w * 256;
      const float* be = sm + L::beta + 8 * w;
      const int c = lane & 7;
      float m[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        float x = 0.f;
#pragma unroll
        for (int j = 0; j < i; ++j) x += (pr[i * 8 + j] + pr[64 + i * 8 + j]) * m[j];
        m[i] = (i == c ? be[c] : 0.f) - be[i] * x;
      }
      if (lane < 8) {
        float* mm = sm + L::mm + w * 128 + c;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          float x = 0.f;
#pragma unroll
          for (int j = 0; j <= i; ++j) x += (pr[128 + i * 8 + j] + pr[192 + i * 8 + j]) * m[j];
          mm[i * 8] = m[i];
          mm[(8 + i) * 8] = x;
        }
      }
    }
    // decay keys and queries from the chunk's start
    if (stager && e8 < L::DP) {
      float* k = sm + L::k + tok * L::DS + e8;
      float c[8], x[8];
      load8(c, sm + L::c + tok * L::DS + e8);
#pragma unroll
      for (int j = 0; j < 8; ++j) c[j] = fast_exp2(c[j]);
      load8(x, k);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] *= c[j];
      store8(k, x);
      load8(x, k + (L::q - L::k));
#pragma unroll
      for (int j = 0; j < 8; ++j) x[j] *= c[j];
      store8(k + (L::q - L::k), x);
    }
    __syncthreads();
    if (owner) {
#pragma unroll
      for (int ch = 0; ch < 2; ++ch) {
        if (t0 + 8 * ch >= n) break;
        const float* row = sm + (col < 8 ? L::k + (8 * ch + col) * L::DS
                                         : L::q + (8 * ch + col - 8) * L::DS) + 4 * g;
        f32x4 acc[2];
        acc[0] = acc[1] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int t = 0; t < DT; ++t) {
          const f32x4 x = *(const f32x4*)(row + 16 * t);
#pragma unroll
          for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int ct = 0; ct < 2; ++ct) acc[ct] = mfma_f32(x[r], st[t][ct][r], acc[ct]);
        }
        // lane groups 0, 1: R of tokens 4 g + r; groups 2, 3: the queries' part of O
        float* vo = sm + L::v + (8 * ch + 4 * (g & 1)) * L::VS + 32 * w + col;
        f32x4 m4 = {0.f, 0.f, 0.f, 0.f};
        if (g < 2) m4 = *(const f32x4*)(sm + L::mm + ch * 128 + col * 8 + 4 * g);
        float* ub = sm + L::tmp + w * 8 * L::UB;
#pragma unroll
        for (int ct = 0; ct < 2; ++ct) {
          f32x4 res;
#pragma unroll
          for (int r = 0; r < 4; ++r)
            res[r] = g < 2 ? vo[r * L::VS + 16 * ct] - acc[ct][r] : 0.f;
          f32x4 y = acc[ct];
          if (g < 2) y = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int r = 0; r < 4; ++r) y = mfma_f32(m4[r], res[r], y);
          if (g < 2) {
#pragma unroll
            for (int r = 0; r < 4; ++r) ub[(4 * g + r) * L::UB + 16 * ct + col] = y[r];
          } else {
#pragma unroll
            for (int r = 0; r < 4; ++r) vo[r * L::VS + 16 * ct] = y[r];
          }
        }
        float u[2][2];
#pragma unroll
        for (int s = 0; s < 2; ++s)
#pragma unroll
          for (int ct = 0; ct < 2; ++ct) u[s][ct] = ub[(4 * s + g) * L::UB + 16 * ct + col];
        const float* gt = sm + L::gt + ch * L::DP + 4 * g;
        const float* kd = sm + L::kd + (8 * ch + g) * L::KD + col;
#pragma unroll
        for (int t = 0; t < DT; ++t) {
          const f32x4 g4 = *(const f32x4*)(gt + 16 * t);
          const float k0 = kd[16 * t], k1 = kd[4 * L::KD + 16 * t];
#pragma unroll
          for (int ct = 0; ct < 2; ++ct) {
            f32x4 x = st[t][ct] * g4;
            x = mfma_f32(k0, u[0][ct], x);
            st[t][ct] = mfma_f32(k1, u[1][ct], x);
          }
        }
      }
    }
    __syncthreads();
    if (stager) {
      float o[NVV][8], so = 0.f;
#pragma unroll
      for (int i = 0; i < NVV; ++i)
        if (128 * i + e8 < a.vdim) {
          load8(o[i], sm + L::v + tok * L::VS + 128 * i + e8);
#pragma unroll
          for (int j = 0; j < 8; ++j) so += o[i][j] * o[i][j];
        }
      const float r = 1.f / sqrtf(sum16(so) / (float)a.vdim + a.eps);
      if (live) {
#pragma unroll
        for (int i = 0; i < NVV; ++i)
          if (128 * i + e8 < a.vdim) {
            float gg[8];
            get(gg, pg[i]);
#pragma unroll
            for (int j = 0; j < 8; ++j) o[i][j] *= r * nw[i][j] * sigmoid_hw(gg[j]);
            store8(out + (int64_t)(row0 + t0 + tok) * ldo + h * a.vdim + 128 * i + e8, o[i]);
          }
      }
      // the next staging overwrites o only with this lane's own v
    }
  }
  if (owner) {
#pragma unroll
    for (int t = 0; t < DT; ++t)
#pragma unroll
      for (int ct = 0; ct < 2; ++ct)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = 16 * t + 4 * g + r, x = 32 * w + 16 * ct + col;
          if (d < a.dim && x < a.vdim) S[(int64_t)d * a.vdim + x] = st[t][ct][r];
        }
  }
  keep_ring<T>(a, slot, h, n, row0, pos0);
}

template <class T, int DPL, int CPL>
__global__ __launch_bounds__(512) void delta_decode_kernel(DeltaArgs a) {
  constexpr int DP = 8 * DPL;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[16];
  const int row = blockIdx.x, h = blockIdx.y;
  const int slot = a.row_state[row];
  const int tid = threadIdx.x, nthr = blockDim.x;
  T* out = (T*)a.out + ((int64_t)row * a.H + h) * a.vdim;
  if (slot < 0) {
    for (int i = tid; i < a.vdim; i += nthr) out[i] = from_f32<T>(0.f);
    return;
  }
  float* ks = sm;
  float* qs = ks + DP;
  float* gs = qs + DP;
  float* vs = gs + DP;
  const int pos = a.positions[row];
  const int lane = tid & 63, p = lane & 7;
  const int col = ((tid >> 6) * 8 + (lane >> 3)) * CPL;
  const int grp = a.H / a.Hk, hk = h / grp;
  const int cq = hk * a.dim, ck = (a.Hk + hk) * a.dim, cv = 2 * a.Hk * a.dim + h * a.vdim;
  float* S = a.state + ((int64_t)slot * a.H + h) * a.dim * a.vdim;
  StateTile<DPL, CPL> st;  // in flight while the token's inputs are prepared
  if (pos > 0) st.load(S, col, p, a.dim, a.vdim);
  else st.zero();

  const T* pr = (const T*)a.proj + (int64_t)row * a.ldp;
  T* ring = (T*)a.ring + (int64_t)slot * a.taps * a.C;
  const bool own = h % grp == 0;
  auto conv = [&](int c, bool keep) {
    const T x0 = pr[c];
    float acc = to_f32(x0) * a.conv_w[(int64_t)(a.taps - 1) * a.C + c];
    const int back = min(pos, a.taps - 1);
    for (int j = 1; j <= back; ++j)
      acc += to_f32(ring[(int64_t)((pos - j) % a.taps) * a.C + c]) *
             a.conv_w[(int64_t)(a.taps - 1 - j) * a.C + c];
    if (keep) ring[(int64_t)(pos % a.taps) * a.C + c] = x0;
    return to_f32(from_f32<T>(silu_as<T>(acc)));
  };
  float sq = 0.f, sk = 0.f, dot = 0.f;
  const float aexp = a.a_exp[h];
  const T* dec = (const T*)a.decay + (int64_t)row * a.ld_decay + h * a.dim;
  for (int i = tid; i < DP; i += nthr) {
    float q = 0.f, k = 0.f, g = 1.f;
    if (i < a.dim) {
      q = conv(cq + i, own);
      k = conv(ck + i, own);
      g = expf(-aexp * softplus_f(to_f32(dec[i]) + a.dt_bias[h * a.dim + i]));
    }
    qs[i] = q;
    ks[i] = k;
    gs[i] = g;
    sq += q * q;
    sk += k * k;
    dot += q * k;
  }
  for (int i = tid; i < a.vdim; i += nthr) vs[i] = conv(cv + i, true);
  const float beta = sigmoid_f(to_f32(pr[a.off_b + h]));
  const float rq = rsqrtf((float)a.dim) / sqrtf(block_sum(sq, red) + 1e-6f);
  const float rk = 1.f / sqrtf(block_sum(sk, red) + 1e-6f);
  const float qk = block_sum(dot, red) * rq * rk;
  for (int i = tid; i < DP; i += nthr) {
    qs[i] *= rq;
    ks[i] *= rk;
  }
  __syncthreads();
  float o[CPL], so = 0.f;
#pragma unroll
  for (int c = 0; c < CPL; ++c) o[c] = 0.f;
  if (col < a.vdim) {
    float v[CPL];
#pragma unroll
    for (int c = 0; c < CPL; ++c) v[c] = col + c < a.vdim ? vs[col + c] : 0.f;
    st.token(ks, qs, gs, p, beta, qk, v, o);
    st.store(S, col, p, a.dim, a.vdim);
#pragma unroll
    for (int c = 0; c < CPL; ++c)
      if (col + c < a.vdim && p == 0) so += o[c] * o[c];
  }
  const float r = 1.f / sqrtf(block_sum(so, red) / (float)a.vdim + a.eps);
  const T* gate = (const T*)a.gate + (int64_t)row * a.ld_gate + h * a.vdim;
  if (p == 0) {
#pragma unroll
    for (int c = 0; c < CPL; ++c)
      if (col + c < a.vdim)
        out[col + c] = from_f32<T>(o[c] * r * a.norm_w[col + c] * sigmoid_f(to_f32(gate[col + c])));
  }
}

template <class T, int DPL, int CPL>
static int scan_go(const DeltaArgs& a, hipStream_t st) {
  using S = ScanShape<DPL>;
  const int waves = (a.vdim + 8 * CPL - 1) / (8 * CPL);
  const int dvp = (a.vdim + 3) & ~3;
  const size_t lds = sizeof(float) * (size_t)(S::CT * (3 * S::DP + 2 * dvp) + 2 * S::CT);
  if (waves > 8 || lds > 65536) return -1;
  delta_scan_kernel<T, DPL, CPL><<<dim3(a.nseg, a.H), dim3(64 * waves), lds, st>>>(a);
  return 0;
}
template <class T, int DPL>
static int scan_c(const DeltaArgs& a, int cpl, hipStream_t st) {
  // columns per lane: at most 8 waves to a workgroup
  if (a.vdim > 256) return scan_go<T, DPL, 8>(a, st);
  if (cpl >= 4 || a.vdim > 128) return scan_go<T, DPL, 4>(a, st);
  return scan_go<T, DPL, 2>(a, st);
}
template <class T>
static int scan_t(const DeltaArgs& a, int cpl, hipStream_t st) {
  const bool big = a.vdim > 256;  // fewer staged tokens
  if (a.dim > 256 || a.vdim > 512) return -1;
  if (a.dim > 128 || big) return scan_c<T, 32>(a, cpl, st);
  if (a.dim > 64) return scan_c<T, 16>(a, cpl, st);
  if (a.dim > 32) return scan_c<T, 8>(a, cpl, st);
  return scan_c<T, 4>(a, cpl, st);
}

template <class T, int DT>
static int chunk_go(const DeltaArgs& a, hipStream_t st) {
  const dim3 grid(a.nseg, a.H);
  if (a.vdim <= 128)
    delta_chunk_kernel<T, DT, 256><<<grid, dim3(256), ChunkLds<DT, 256>::BYTES, st>>>(a);
  else
    delta_chunk_kernel<T, DT, 512><<<grid, dim3(512), ChunkLds<DT, 512>::BYTES, st>>>(a);
  static_assert(ChunkLds<DT, 512>::BYTES <= 65536, "LDS without an attribute");
  return 0;
}
template <class T>
static int chunk_t(const DeltaArgs& a, hipStream_t st) {
  if (a.dim <= 32) return chunk_go<T, 2>(a, st);
  if (a.dim <= 64) return chunk_go<T, 4>(a, st);
  return chunk_go<T, 8>(a, st);
}

// cpl 0: the chunk form where the sizes allow it
int launch_delta_scan(int f32, const DeltaArgs& a, int cpl, hipStream_t st) {
  if (a.nseg == 0) return 0;
  if (a.Hk < 1 || a.H % a.Hk) return -1;
  if (cpl == 0) {
    if (a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= 128 && a.vdim <= 256 &&
        a.ld_decay % 8 == 0 && a.ld_gate % 8 == 0) {
      const int rc = f32 ? chunk_t<float>(a, st) : chunk_t<bf16_t>(a, st);
      return rc ? rc : (int)hipGetLastError();
    }
    cpl = 4;
  }
  const int rc = f32 ? scan_t<float>(a, cpl, st) : scan_t<bf16_t>(a, cpl, st);
  return rc ? rc : (int)hipGetLastError();
}

template <class T, int DPL, int CPL>
static int decode_go(const DeltaArgs& a, hipStream_t st) {
  const int waves = (a.vdim + 8 * CPL - 1) / (8 * CPL);
  const size_t lds = sizeof(float) * (size_t)(3 * 8 * DPL + a.vdim);
  if (waves > 8) return -1;
  delta_decode_kernel<T, DPL, CPL><<<dim3(a.rows, a.H), dim3(64 * waves), lds, st>>>(a);
  return 0;
}
template <class T, int DPL>
static int decode_c(const DeltaArgs& a, hipStream_t st) {
  return a.vdim > 256 ? decode_go<T, DPL, 8>(a, st) : decode_go<T, DPL, 4>(a, st);
}
template <class T>
static int decode_t(const DeltaArgs& a, hipStream_t st) {
  if (a.dim > 256 || a.vdim > 512) return -1;
  if (a.dim > 128) return decode_c<T, 32>(a, st);
  if (a.dim > 64) return decode_c<T, 16>(a, st);
  if (a.dim > 32) return decode_c<T, 8>(a, st);
  return decode_c<T, 4>(a, st);
}

int launch_delta_decode(int f32, const DeltaArgs& a, hipStream_t st) {
  if (a.rows == 0) return 0;
  if (a.Hk < 1 || a.H % a.Hk) return -1;
  const int rc = f32 ? decode_t<float>(a, st) : decode_t<bf16_t>(a, st);
  return rc ? rc : (int)hipGetLastError();
}

}  // namespace drtc
