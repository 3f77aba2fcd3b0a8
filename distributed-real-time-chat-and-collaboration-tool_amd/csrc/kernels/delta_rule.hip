// Gated delta rule with per-channel decay (gfx950): short causal convolutions, the recurrence,
// and the gated output norm.
//
// Per head, with the 32-bit state S [dim, vdim] of a sequence:
//   S <- g * S (rows),  u = beta (v - S^T k),  S <- S + k u^T,  o = S^T q
//   out = o / rms(o) * w * sigmoid(gate)
// The columns of S are independent, so a column lives in the registers of one quad of lanes:
// lane 4 c + p of a wave holds rows {16 m + 4 p .. + 3} of CPL columns, both products with the
// decayed state are taken in one pass (S^T q = (gS)^T q + u (k.q)) and reduced over the quad
// with two DPP adds.
//   short_conv_kernel    prompt portions: convolution + SiLU of the packed rows; inputs ahead
//                        of a portion come from the sequence's ring of the last `taps` inputs
//   delta_scan_kernel    one workgroup per (portion, head): unit norms, decays and gates of CT
//                        tokens at a time staged in LDS, then their recurrence
//   delta_decode_kernel  one workgroup per (sequence, head): all of it for one token; the
//                        state streams through registers once
// A ring entry is position % taps: the entry a token writes is the one its own convolution no
// longer reads, so heads sharing a key never race on it.
#include "hybrid_launchers.h"
#include "typed.h"

#include <algorithm>

namespace drtc {

DRTC_DEVICE float silu_f(float x) { return x / (1.f + expf(-x)); }
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
  for (int row = blockIdx.x * kConvRows; row < r1; ++row) {
    const int slot = row_state[row];
    float acc[VEC];
#pragma unroll
    for (int i = 0; i < VEC; ++i) acc[i] = 0.f;
    if (slot >= 0) {
      const int off = row_off[row], pos = positions[row];
      auto tap = [&](int j, const float (&wj)[VEC]) {  // j tokens back
        float x[VEC];
        if (j <= off) loadx(x, proj + (int64_t)(row - j) * ldp + c);
        else if (j <= pos) loadx(x, ring + ((int64_t)slot * taps + (pos - j) % taps) * C + c);
        else return;
#pragma unroll
        for (int i = 0; i < VEC; ++i) acc[i] += x[i] * wj[i];
      };
      if constexpr (TAPS != 0) {
#pragma unroll
        for (int j = 0; j < TAPS; ++j) tap(j, wr[TAPS - 1 - j]);
      } else {
        for (int j = 0; j < taps; ++j) {
          loadw(wr[0], taps - 1 - j);
          tap(j, wr[0]);
        }
      }
#pragma unroll
      for (int i = 0; i < VEC; ++i) acc[i] = silu_f(acc[i]);
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
  DRTC_DEVICE static int row_of(int i, int p) { return 16 * (i >> 2) + 4 * p + (i & 3); }
  DRTC_DEVICE void load(const float* S, int col, int p, int dim, int vdim) {
    if (CPL == 4 && (vdim & 3) == 0) {
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int r = row_of(i, p);
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (r < dim && col < vdim) v = *reinterpret_cast<const f32x4*>(S + (int64_t)r * vdim + col);
#pragma unroll
        for (int c = 0; c < CPL; ++c) s[i][c] = v[c & 3];
      }
      return;
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
    if (CPL == 4 && (vdim & 3) == 0) {
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int r = row_of(i, p);
        f32x4 v;
#pragma unroll
        for (int c = 0; c < 4; ++c) v[c] = s[i][c % CPL];
        if (r < dim && col < vdim) *reinterpret_cast<f32x4*>(S + (int64_t)r * vdim + col) = v;
      }
      return;
    }
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int r = row_of(i, p);
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        if (r < dim && col + c < vdim) S[(int64_t)r * vdim + col + c] = s[i][c];
    }
  }
  // One token: k, q, g rows in LDS (padded to 4 DPL), qk = k.q; o[c] = the read-out.
  DRTC_DEVICE void token(const float* k, const float* q, const float* g, int p, float beta,
                         float qk, const float (&v)[CPL], float (&o)[CPL]) {
    float kk[DPL], ks[CPL], qs[CPL];
#pragma unroll
    for (int c = 0; c < CPL; ++c) ks[c] = qs[c] = 0.f;
#pragma unroll
    for (int m = 0; m < DPL / 4; ++m) {
      const int at = 16 * m + 4 * p;
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
      const float u = beta * (v[c] - quad_sum(ks[c]));
      o[c] = quad_sum(qs[c]) + u * qk;
#pragma unroll
      for (int i = 0; i < DPL; ++i) s[i][c] += kk[i] * u;
    }
  }
};

template <int DPL>
struct ScanShape {
  static constexpr int DP = 4 * DPL;           // padded key size
  static constexpr int CT = DPL <= 32 ? 16 : 8;  // tokens staged at a time
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

  const int lane = tid & 63, p = lane & 3;
  const int col = ((tid >> 6) * 16 + (lane >> 2)) * CPL;
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
  // convolution inputs of the last `taps` tokens
  T* ring = (T*)a.ring + (int64_t)slot * a.taps * a.C;
  const int nr = min(n, a.taps), own = h % grp == 0 ? 2 * a.dim : 0;
  for (int k = tid; k < nr * (own + a.vdim); k += nthr) {
    const int j = k / (own + a.vdim), i = k % (own + a.vdim);
    const int c = i < own ? (i < a.dim ? cq + i : ck + i - a.dim) : cv + i - own;
    const int t = n - nr + j;
    ring[(int64_t)((pos0 + t) % a.taps) * a.C + c] = proj[(int64_t)(row0 + t) * a.ldp + c];
  }
}

template <class T, int DPL, int CPL>
__global__ __launch_bounds__(512) void delta_decode_kernel(DeltaArgs a) {
  constexpr int DP = 4 * DPL;
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
  const int lane = tid & 63, p = lane & 3;
  const int col = ((tid >> 6) * 16 + (lane >> 2)) * CPL;
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
    return to_f32(from_f32<T>(silu_f(acc)));
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
  const int waves = (a.vdim + 16 * CPL - 1) / (16 * CPL);
  const int dvp = (a.vdim + 3) & ~3;
  const size_t lds = sizeof(float) * (size_t)(S::CT * (3 * S::DP + 2 * dvp) + 2 * S::CT);
  if (waves > 8 || lds > 65536) return -1;
  delta_scan_kernel<T, DPL, CPL><<<dim3(a.nseg, a.H), dim3(64 * waves), lds, st>>>(a);
  return 0;
}
template <class T, int DPL>
static int scan_c(const DeltaArgs& a, int cpl, hipStream_t st) {
  // columns per lane: at most 8 waves to a workgroup
  if (cpl >= 4 || a.vdim > 256) return scan_go<T, DPL, 4>(a, st);
  if (cpl >= 2 || a.vdim > 128) return scan_go<T, DPL, 2>(a, st);
  return scan_go<T, DPL, 1>(a, st);
}
template <class T>
static int scan_t(const DeltaArgs& a, int cpl, hipStream_t st) {
  const bool big = a.vdim > 256;  // fewer staged tokens
  if (a.dim > 256 || a.vdim > 512) return -1;
  if (a.dim > 128 || big) return scan_c<T, 64>(a, cpl, st);
  if (a.dim > 64) return scan_c<T, 32>(a, cpl, st);
  if (a.dim > 32) return scan_c<T, 16>(a, cpl, st);
  return scan_c<T, 8>(a, cpl, st);
}

int launch_delta_scan(int f32, const DeltaArgs& a, int cpl, hipStream_t st) {
  if (a.nseg == 0) return 0;
  if (a.Hk < 1 || a.H % a.Hk) return -1;
  const int rc = f32 ? scan_t<float>(a, cpl, st) : scan_t<bf16_t>(a, cpl, st);
  return rc ? rc : (int)hipGetLastError();
}

template <class T, int DPL, int CPL>
static int decode_go(const DeltaArgs& a, hipStream_t st) {
  const int waves = (a.vdim + 16 * CPL - 1) / (16 * CPL);
  const size_t lds = sizeof(float) * (size_t)(3 * 4 * DPL + a.vdim);
  if (waves > 8) return -1;
  delta_decode_kernel<T, DPL, CPL><<<dim3(a.rows, a.H), dim3(64 * waves), lds, st>>>(a);
  return 0;
}
template <class T>
static int decode_t(const DeltaArgs& a, hipStream_t st) {
  if (a.dim > 256 || a.vdim > 512) return -1;
  if (a.dim > 128)
    return a.vdim > 256 ? decode_go<T, 64, 4>(a, st) : decode_go<T, 64, 2>(a, st);
  if (a.dim > 64) return decode_go<T, 32, 4>(a, st);
  if (a.dim > 32) return decode_go<T, 16, 4>(a, st);
  return decode_go<T, 8, 4>(a, st);
}

int launch_delta_decode(int f32, const DeltaArgs& a, hipStream_t st) {
  if (a.rows == 0) return 0;
  if (a.Hk < 1 || a.H % a.Hk) return -1;
  const int rc = f32 ? decode_t<float>(a, st) : decode_t<bf16_t>(a, st);
  return rc ? rc : (int)hipGetLastError();
}

}  // namespace drtc
