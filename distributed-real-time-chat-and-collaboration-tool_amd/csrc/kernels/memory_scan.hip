// Linear attention with a matrix state per head (gfx950): retention and the mLSTM.
//
// Per head, with the 32-bit state S [dim, vdim] of a sequence:
//   S <- a S + b k v^T,  o = S^T q,  out = o / rms(o) * w * gate
// where a is a fixed decay and b = 1 (retention), or, with log gates f <= 0 and i of the token and
// a running maximum m <- max(f + m, i) from m = 0 on, a = e^(f + m_old - m), b = e^(i - m); a
// normaliser n <- a n + b k then divides the read-out, o / (max(|n.q|, e^-m) + 1e-6) (mLSTM).
// Queries and keys may be rotated (pairs half the rotated part apart) on their way in.
//
//   memory_chunk_kernel   prompt portions on MFMA, 64 tokens at a time (derivation at the kernel);
//                         bf16 only
//   memory_scan_kernel    the same token by token: fp32, and sizes the chunk form does not take
//   memory_decode_kernel  one workgroup per (sequence, head): all of it for one token; the state
//                         streams through registers once
//   memory_finish_kernel  norm and gate of heads too wide for one workgroup (slices > 1); every
//                         slice keeps its own copy of n and m, so that no order between them is
//                         needed
#include "hybrid_launchers.h"
#include "typed.h"

#include <algorithm>

namespace drtc {

DRTC_DEVICE float mem_sigmoid(float x) { return 1.f / (1.f + expf(-x)); }
// log sigmoid(x) = -log(1 + e^-x)
DRTC_DEVICE float mem_logsig(float x) { return x < -15.f ? x : -log1pf(expf(-x)); }
// read-out gate
template <class T>
DRTC_DEVICE float mem_gate(float g, int silu) {
  float s;
  if constexpr (sizeof(T) == 2) s = __builtin_amdgcn_rcpf(1.f + fast_exp2(-kLog2e * g));
  else s = mem_sigmoid(g);
  return silu ? g * s : s;
}

// log gates of a head's token
template <class T>
DRTC_DEVICE void mem_gates(const MemoryArgs& a, const T* row, int h, float& f, float& i) {
  if (a.log_decay) {
    f = a.log_decay[h];
    i = 0.f;
  } else {
    i = a.cap * tanhf((to_f32(row[a.off_i + h]) + a.i_bias[h]) / a.cap);
    f = mem_logsig(a.cap * tanhf((to_f32(row[a.off_f + h]) + a.f_bias[h]) / a.cap));
  }
}

// Element c of a head's query or key, rotated and scaled.
template <class T>
DRTC_DEVICE float mem_turned(const T* x, int c, const float* cs, int rot, float scale) {
  const int half = rot >> 1;
  float y = to_f32(x[c]);
  if (c < half) y = y * cs[c] - to_f32(x[c + half]) * cs[half + c];
  else if (c < rot) y = y * cs[c - half] + to_f32(x[c - half]) * cs[c];
  return y * scale;
}

// ------------------------------------------------------------------ token by token
// A column of S lives in 8 lanes, lane p of them holds rows {32 m + 4 p .. + 3}; CPL columns to a
// lane.  One more group of 8 lanes keeps the normaliser, as a column whose value is always 1.
template <int DPL>
DRTC_DEVICE int mem_row(int i, int p) { return 32 * (i >> 2) + 4 * p + (i & 3); }

template <int DPL>
struct MemShape {
  static constexpr int DP = 8 * DPL;             // padded key size
  static constexpr int CT = DPL <= 16 ? 16 : 8;  // tokens staged at a time
};

template <class T, int DPL, int CPL>
__global__ __launch_bounds__(576) void memory_scan_kernel(MemoryArgs a) {
  constexpr int DP = MemShape<DPL>::DP, CT = MemShape<DPL>::CT;
  extern __shared__ __attribute__((aligned(16))) float ms[];
  const int seg = blockIdx.x, h = blockIdx.y, sl = blockIdx.z;
  const int slot = a.seg_state[seg];
  const int n = a.seg_len[seg], row0 = a.seg_row[seg], pos0 = a.seg_pos[seg];
  const int tid = threadIdx.x, nthr = blockDim.x;
  const int c0 = a.slices > 1 ? sl * 128 : 0;
  const int cols = a.slices > 1 ? min(128, a.vdim - c0) : a.vdim, cp = (cols + 3) & ~3;
  T* out = (T*)a.out;
  if (slot < 0) {
    for (int i = tid; i < n * cols; i += nthr)
      out[(int64_t)(row0 + i / cols) * a.ldo + h * a.vdim + c0 + i % cols] = from_f32<T>(0.f);
    return;
  }
  const bool gated = a.log_decay == nullptr;
  float* ks = ms;
  float* qs = ks + CT * DP;
  float* vs = qs + CT * DP;
  float* os = vs + CT * cp;
  float* av = os + CT * cp;  // decay, input weight, n.q, e^-m of the staged tokens
  float* bv = av + CT;
  float* nq = bv + CT;
  float* em = nq + CT;

  const int lane = tid & 63, p = lane & 7, grp = tid >> 3;
  const int groups = (cols + CPL - 1) / CPL;
  const bool norm = gated && grp == groups, live = grp < groups || norm;
  const int col = grp * CPL;
  float* S = a.state + ((int64_t)slot * a.H + h) * a.dim * a.vdim + c0;
  float* N = gated ? a.nrm + (((int64_t)slot * a.H + h) * a.slices + sl) * a.dim : nullptr;
  float* top = gated ? a.top + ((int64_t)slot * a.H + h) * a.slices + sl : nullptr;
  float s[DPL][CPL];
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int r = mem_row<DPL>(i, p);
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      s[i][c] = 0.f;
      if (pos0 > 0 && live && r < a.dim) {
        if (norm) s[i][c] = c == 0 ? N[r] : 0.f;
        else if (col + c < cols) s[i][c] = S[(int64_t)r * a.vdim + col + c];
      }
    }
  }
  float m = gated && pos0 > 0 ? top[0] : 0.f;
  const int l16 = tid & 15, g16 = tid >> 4, n16 = nthr >> 4;
  const T* proj = (const T*)a.proj;

  for (int t0 = 0; t0 < n; t0 += CT) {
    const int nt = min(CT, n - t0);
    for (int t = g16; t < nt; t += n16) {  // 16 lanes per token
      const T* pr = proj + (int64_t)(row0 + t0 + t) * a.ldp;
      const float* cs = a.rot_dims ? a.cos_sin + (int64_t)(pos0 + t0 + t) * a.rot_dims : nullptr;
      for (int i = l16; i < DP; i += 16) {
        qs[t * DP + i] = i < a.dim ? mem_turned(pr + h * a.dim, i, cs, a.rot_dims, a.q_scale) : 0.f;
        ks[t * DP + i] =
            i < a.dim ? mem_turned(pr + a.off_k + h * a.dim, i, cs, a.rot_dims, a.k_scale) : 0.f;
      }
      for (int i = l16; i < cols; i += 16) vs[t * cp + i] = to_f32(pr[a.off_v + h * a.vdim + c0 + i]);
      if (l16 == 0) {
        float f, i;
        mem_gates(a, pr, h, f, i);
        av[t] = f;
        bv[t] = i;
      }
    }
    __syncthreads();
    // every thread follows m; the first leaves decays and weights behind
    float mm = m, da[CT], db[CT];
#pragma unroll
    for (int t = 0; t < CT; ++t) {
      if (t >= nt) break;
      const float f = av[t], i = bv[t], mn = fmaxf(f + mm, i);
      da[t] = expf(f + mm - mn);
      db[t] = expf(i - mn);
      mm = mn;
      if (tid == 0) em[t] = expf(-mn);
    }
    m = mm;
    if (live) {
#pragma unroll
      for (int t = 0; t < CT; ++t) {
        if (t >= nt) break;
        float u[CPL], o[CPL];
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
          u[c] = norm ? (c == 0 ? db[t] : 0.f) : col + c < cols ? db[t] * vs[t * cp + col + c] : 0.f;
          o[c] = 0.f;
        }
#pragma unroll
        for (int j = 0; j < DPL / 4; ++j) {
          const f32x4 k4 = *reinterpret_cast<const f32x4*>(ks + t * DP + 32 * j + 4 * p);
          const f32x4 q4 = *reinterpret_cast<const f32x4*>(qs + t * DP + 32 * j + 4 * p);
#pragma unroll
          for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int c = 0; c < CPL; ++c) {
              const float x = s[4 * j + r][c] * da[t] + k4[r] * u[c];
              s[4 * j + r][c] = x;
              o[c] += q4[r] * x;
            }
        }
#pragma unroll
        for (int c = 0; c < CPL; ++c) {
          const float x = sum8(o[c]);
          if (p == 0) {
            if (norm) {
              if (c == 0) nq[t] = x;
            } else if (col + c < cols) {
              os[t * cp + col + c] = x;
            }
          }
        }
      }
    }
    __syncthreads();
    for (int t = g16; t < nt; t += n16) {
      const int64_t row = row0 + t0 + t;
      const float inv = gated ? 1.f / (fmaxf(fabsf(nq[t]), em[t]) + 1e-6f) : 1.f;
      float so = 0.f;
      for (int i = l16; i < cols; i += 16) {
        const float o = os[t * cp + i] * inv;
        so += o * o;
      }
      so = sum16(so);
      T* op = out + row * a.ldo + h * a.vdim + c0;
      const float r = inv / sqrtf(so / (float)a.vdim + a.eps);
      const T* gp = proj + row * a.ldp + a.off_g + h * a.vdim;
      for (int i = l16; i < cols; i += 16) {
        const float o = os[t * cp + i];
        if (a.slices > 1) op[i] = from_f32<T>(o * inv);
        else
          op[i] = from_f32<T>(o * r * (a.norm_w ? a.norm_w[h * a.vdim + i] : 1.f) *
                              mem_gate<T>(to_f32(gp[i]), a.silu));
      }
    }
    __syncthreads();
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int r = mem_row<DPL>(i, p);
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        if (r >= a.dim) continue;
        if (norm) {
          if (c == 0) N[r] = s[i][c];
        } else if (col + c < cols) {
          S[(int64_t)r * a.vdim + col + c] = s[i][c];
        }
      }
    }
  }
  if (gated && tid == 0) top[0] = m;
}

// ------------------------------------------------------------------ chunks on MFMA
// For the tokens t = 0..63 of a chunk let F_t be the running sum of f (log2), g_t = i_t - F_t,
// M_t = max(m_0, g_0 .. g_t): then m_t = F_t + M_t, and unrolling the recurrence from the state S
// scaled by 2^-m_0,
//   o_t  = 2^(m_0 - M_t) S^T q_t + sum_{j <= t} P_tj v_j,  P_tj = (q_t . k_j) 2^(g_j - M_t)
//   S   <- 2^(m_0 - M_63) S + sum_j 2^(g_j - M_63) k_j v_j^T
// and n likewise with v = 1; no exponent is positive.  A wave keeps 16 CT columns of S as
// accumulator tiles.  Their layout (row 4 g + r of lane group g) is that of an A operand of S^T
// whose k-step takes dims 4 g + r of two tiles, so S feeds O^T = S^T Q^T without lane movement,
// split into two bf16 parts (16 significant bits).  K and V are read transposed from LDS; the
// weights of the update go onto the V fragments in registers.
constexpr int kMC = 64;

typedef short mem_s16x4 __attribute__((ext_vector_type(4)));
DRTC_DEVICE bf16x4 mem_read_tr16(const bf16_t* p) {
  mem_s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) mem_s16x4*)(p));
  return __builtin_bit_cast(bf16x4, v);
}
DRTC_DEVICE bf16x8 mem_join(bf16x4 lo, bf16x4 hi) {
  bf16x8 v;
#pragma unroll
  for (int j = 0; j < 4; ++j) { v[j] = lo[j]; v[4 + j] = hi[j]; }
  return v;
}
DRTC_DEVICE bf16x8 mem_zero8() {
  bf16x8 z;
#pragma unroll
  for (int j = 0; j < 8; ++j) z[j] = f2bf(0.f);
  return z;
}
DRTC_DEVICE float lane_scan_sum(float v, int lane) {
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float u = __shfl_up(v, o, 64);
    if (lane >= o) v += u;
  }
  return v;
}
DRTC_DEVICE float lane_scan_max(float v, int lane) {
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float u = __shfl_up(v, o, 64);
    if (lane >= o) v = fmaxf(v, u);
  }
  return v;
}

// KS: 32-dim steps of a key (padded); NW waves of CT column tiles
template <int KS, int NW, int CT>
struct MemLds {
  static constexpr int DP = 32 * KS, COLS = 16 * CT * NW;
  static constexpr int QROW = DP + 8, KROW = DP + 16, VROW = COLS + 16, PROW = kMC + 8;
  // bf16 elements, then floats
  static constexpr int q = 0, k = q + kMC * QROW, v = k + kMC * KROW, p = v + kMC * VROW;
  static constexpr int bf = p + kMC * PROW;
  static constexpr int n = 0, g = n + DP, m = g + kMC, in = m + kMC, em = in + kMC, w = em + kMC;
  static constexpr int qn = w + kMC, rs = qn + kMC, ss = rs + 2 * kMC, fl = ss + NW * kMC;
  static constexpr size_t BYTES = (size_t)bf * 2 + (size_t)fl * 4;
};

template <int KS, int NW, int CT, bool GATED>
__global__ __launch_bounds__(64 * NW, 2) void memory_chunk_kernel(MemoryArgs a) {
  using L = MemLds<KS, NW, CT>;
  constexpr int NTHR = 64 * NW, PU = L::DP / 16, NU = (kMC * PU + NTHR - 1) / NTHR, NV = 2 * CT;
  extern __shared__ __attribute__((aligned(16))) bf16_t mb[];
  float* fl = reinterpret_cast<float*>(mb + L::bf);
  const int seg = blockIdx.x, h = blockIdx.y, sl = blockIdx.z, c0 = sl * L::COLS;
  const int slot = a.seg_state[seg];
  const int n = a.seg_len[seg], row0 = a.seg_row[seg], pos0 = a.seg_pos[seg];
  const int tid = threadIdx.x, w = wave_id_uniform(), lane = tid & 63, col = lane & 15, g = lane >> 4;
  bf16_t* out = (bf16_t*)a.out + h * a.vdim;
  if (slot < 0) {
    const int cols = min(L::COLS, a.vdim - c0);
    for (int i = tid; i < n * cols; i += NTHR)
      out[(int64_t)(row0 + i / cols) * a.ldo + c0 + i % cols] = f2bf(0.f);
    return;
  }
  const bf16_t* proj = (const bf16_t*)a.proj + (int64_t)row0 * a.ldp;
  const int cw = c0 + 16 * CT * w;  // this wave's first column
  float* S = a.state + ((int64_t)slot * a.H + h) * a.dim * a.vdim;
  float* N = GATED ? a.nrm + (((int64_t)slot * a.H + h) * a.slices + sl) * a.dim : nullptr;
  float* top = GATED ? a.top + ((int64_t)slot * a.H + h) * a.slices + sl : nullptr;

  f32x4 st[2 * KS][CT];
#pragma unroll
  for (int t = 0; t < 2 * KS; ++t)
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * t + 4 * g + r, x = cw + 16 * ct + col;
        st[t][ct][r] = pos0 > 0 && d < a.dim && x < a.vdim ? S[(int64_t)d * a.vdim + x] : 0.f;
      }
  float m0 = 0.f;  // log2 units
  if constexpr (GATED) {
    if (pos0 > 0) m0 = top[0] * kLog2e;
    for (int d = tid; d < L::DP; d += NTHR) fl[L::n + d] = pos0 > 0 && d < a.dim ? N[d] : 0.f;
  }
  const float f2 = GATED ? 0.f : a.log_decay[h] * kLog2e;
  f32x4 nw[CT];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int x = cw + 16 * ct + 4 * g + r;
      nw[ct][r] = a.norm_w && x < a.vdim ? a.norm_w[h * a.vdim + x] : 1.f;
    }

  // staging: a unit is two 8-element vectors of a token's query and key - the two halves of eight
  // rotated pairs, or neighbours behind the rotated part
  const int half = a.rot_dims >> 1;
  auto unit = [&](int i, int& tok, int& e0, int& e1, bool& turn) {
    const int u = tid + i * NTHR;
    tok = u / PU;
    const int pr = u % PU;
    turn = 16 * pr < a.rot_dims;
    e0 = turn ? 8 * pr : 16 * pr;
    e1 = turn ? 8 * pr + half : 16 * pr + 8;
    return u < kMC * PU;
  };
  bf16x8 pq[NU][2], pk[NU][2], pv[NV];
  float gi = 0.f, gf = 0.f;
  auto prefetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < NU; ++i) {
      int tok, e0, e1;
      bool turn;
      const bool in = unit(i, tok, e0, e1, turn) && t0 + tok < n;
      const bf16_t* r = proj + (int64_t)(t0 + tok) * a.ldp + h * a.dim;
      const bool in0 = in && e0 < a.dim, in1 = in && e1 < a.dim;
      pq[i][0] = in0 ? load_bf16x8(r + e0) : mem_zero8();
      pq[i][1] = in1 ? load_bf16x8(r + e1) : mem_zero8();
      pk[i][0] = in0 ? load_bf16x8(r + a.off_k + e0) : mem_zero8();
      pk[i][1] = in1 ? load_bf16x8(r + a.off_k + e1) : mem_zero8();
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = tid + i * NTHR, tok = v / (L::COLS / 8), c = c0 + (v % (L::COLS / 8)) * 8;
      pv[i] = t0 + tok < n && c < a.vdim
          ? load_bf16x8(proj + (int64_t)(t0 + tok) * a.ldp + a.off_v + h * a.vdim + c) : mem_zero8();
    }
    if (GATED && t0 + lane < n) {
      const bf16_t* r = proj + (int64_t)(t0 + lane) * a.ldp + h;
      gi = bf2f(r[a.off_i]);
      gf = bf2f(r[a.off_f]);
    }
  };
  prefetch(0);
  const int tr_k = ((col >> 2) + 4 * g) * L::KROW + 4 * (col & 3);
  const int tr_v = ((col >> 2) + 4 * g) * L::VROW + 4 * (col & 3) + 16 * CT * w;
  const float ib = GATED ? a.i_bias[h] : 0.f, fb = GATED ? a.f_bias[h] : 0.f;

  for (int t0 = 0; t0 < n; t0 += kMC) {
    const int nt = min(kMC, n - t0);
    // gates: one token to a lane, every wave for itself
    float F, gg, M;
    if constexpr (GATED) {
      const float i = a.cap * tanhf((gi + ib) / a.cap), f = mem_logsig(a.cap * tanhf((gf + fb) / a.cap));
      F = lane_scan_sum(lane < nt ? f * kLog2e : 0.f, lane);
      gg = lane < nt ? i * kLog2e - F : kNegBig;
      M = fmaxf(m0, lane_scan_max(gg, lane));
    } else {
      F = (float)min(lane + 1, nt) * f2;
      gg = -F;
      M = -F;
    }
    const float M1 = __shfl(M, 63, 64), gamma = fast_exp2(m0 - M1);
    if (w == 0) {
      fl[L::g + lane] = gg;
      fl[L::m + lane] = M;
      fl[L::in + lane] = fast_exp2(m0 - M);
      fl[L::em + lane] = fast_exp2(-(F + M));
      fl[L::w + lane] = lane < nt ? fast_exp2(gg - M1) : 0.f;
    }
    if constexpr (GATED) m0 = __shfl(F, 63, 64) + M1;
#pragma unroll
    for (int i = 0; i < NU; ++i) {
      int tok, e0, e1;
      bool turn;
      if (!unit(i, tok, e0, e1, turn)) continue;
      float x[2][8], y[2][8];
#pragma unroll
      for (int j = 0; j < 8; ++j)
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          x[e][j] = bf2f(pq[i][e][j]);
          y[e][j] = bf2f(pk[i][e][j]);
        }
      if (turn && t0 + tok < n) {
        const float* cs = a.cos_sin + (int64_t)(pos0 + t0 + tok) * a.rot_dims + e0;
        float c[8], s[8];
        load8(c, cs);
        load8(s, cs + half);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float u = x[0][j], v = x[1][j], z = y[0][j], zz = y[1][j];
          x[0][j] = u * c[j] - v * s[j];
          x[1][j] = v * c[j] + u * s[j];
          y[0][j] = z * c[j] - zz * s[j];
          y[1][j] = zz * c[j] + z * s[j];
        }
      }
      // columns behind the head (and, unrotated, their vectors) are zeros
#pragma unroll
      for (int e = 0; e < 2; ++e) {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          x[e][j] *= a.q_scale;
          y[e][j] *= a.k_scale;
        }
        const int at = e ? e1 : e0;
        store8(mb + L::q + tok * L::QROW + at, x[e]);
        store8(mb + L::k + tok * L::KROW + at, y[e]);
      }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = tid + i * NTHR;
      store_bf16x8(mb + L::v + (v / (L::COLS / 8)) * L::VROW + (v % (L::COLS / 8)) * 8, pv[i]);
    }
    prefetch(t0 + kMC);
    __syncthreads();

    // weighted scores of 16 tokens to a wave (8 waves: every other key tile each)
    {
      const int tt = w & 3, t = 16 * tt + col;
      const float Mt = fl[L::m + t];
      bf16x8 qf[KS];
#pragma unroll
      for (int s = 0; s < KS; ++s) qf[s] = load_bf16x8(mb + L::q + t * L::QROW + 32 * s + 8 * g);
      float rsum = 0.f;
#pragma unroll
      for (int st_ = 0; st_ < 4; ++st_) {
        if (NW == 8 && (st_ & 1) != (w >> 2)) continue;
        if (st_ > (tt | 1)) continue;
        bf16x4 pf;
#pragma unroll
        for (int r = 0; r < 4; ++r) pf[r] = f2bf(0.f);
        if (st_ <= tt) {
          f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int s = 0; s < KS; ++s)
            sc = mfma16(load_bf16x8(mb + L::k + (16 * st_ + col) * L::KROW + 32 * s + 8 * g), qf[s], sc);
          const f32x4 gj = *reinterpret_cast<const f32x4*>(fl + L::g + 16 * st_ + 4 * g);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float p = 16 * st_ + 4 * g + r <= t ? sc[r] * fast_exp2(fminf(gj[r] - Mt, 0.f)) : 0.f;
            rsum += p;
            pf[r] = f2bf(p);
          }
        }
        // keys in the order of the V fragments: 4 g + r of both tiles of a 32-key step together
        *reinterpret_cast<bf16x4*>(mb + L::p + t * L::PROW + 32 * (st_ >> 1) + 8 * g + 4 * (st_ & 1)) = pf;
      }
      if constexpr (GATED) {
        rsum += __shfl_xor(rsum, 16, 64);
        rsum += __shfl_xor(rsum, 32, 64);
        if (g == 0) fl[L::rs + (w >> 2) * kMC + t] = rsum;
        constexpr int PART = L::DP / NW;  // n.q: NW lanes to a token
        const int tok = tid / NW, part = tid % NW;
        float d = 0.f;
#pragma unroll
        for (int j = 0; j < PART; j += 4) {
          const bf16x4 q4 = load_bf16x4(mb + L::q + tok * L::QROW + part * PART + j);
          const f32x4 n4 = *reinterpret_cast<const f32x4*>(fl + L::n + part * PART + j);
#pragma unroll
          for (int r = 0; r < 4; ++r) d += bf2f(q4[r]) * n4[r];
        }
        d = NW == 4 ? quad_sum(d) : sum8(d);
        if (part == 0) fl[L::qn + tok] = d;
      }
    }
    __syncthreads();

    bf16x4 gate[CT][4];
    if (a.slices == 1) {
#pragma unroll
      for (int ct = 0; ct < CT; ++ct)
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
          const int t = 16 * tt + col, x = cw + 16 * ct + 4 * g;
          if (t < nt && x < a.vdim)
            gate[ct][tt] = load_bf16x4(proj + (int64_t)(t0 + t) * a.ldp + a.off_g + h * a.vdim + x);
        }
    }
    f32x4 o[CT][4];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) o[ct][tt] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      bf16x8 qf[4];
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        const bf16_t* q = mb + L::q + (16 * tt + col) * L::QROW + 32 * s + 4 * g;
        qf[tt] = mem_join(load_bf16x4(q), load_bf16x4(q + 16));
      }
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        bf16x8 hi, lo;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float x = st[2 * s + (j >> 2)][ct][j & 3];
          hi[j] = f2bf(x);
          lo[j] = f2bf(x - bf2f(hi[j]));
        }
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
          o[ct][tt] = mfma16(hi, qf[tt], o[ct][tt]);
          o[ct][tt] = mfma16(lo, qf[tt], o[ct][tt]);
        }
      }
    }
    float inv[4];
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) {
      const int t = 16 * tt + col;
      const float in = fl[L::in + t];
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) o[ct][tt] *= in;
      inv[tt] = 1.f;
      if constexpr (GATED) {
        float d = in * fl[L::qn + t] + fl[L::rs + t];
        if constexpr (NW == 8) d += fl[L::rs + kMC + t];
        inv[tt] = 1.f / (fmaxf(fabsf(d), fl[L::em + t]) + 1e-6f);
      }
    }
    bf16x8 vw[2][CT], wf[2];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      const f32x4 w0 = *reinterpret_cast<const f32x4*>(fl + L::w + 32 * ks + 4 * g);
      const f32x4 w1 = *reinterpret_cast<const f32x4*>(fl + L::w + 32 * ks + 16 + 4 * g);
      bf16x8 vf[CT];
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        const bf16_t* v = mb + L::v + tr_v + 32 * ks * L::VROW + 16 * ct;
        vf[ct] = mem_join(mem_read_tr16(v), mem_read_tr16(v + 16 * L::VROW));
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          vw[ks][ct][j] = f2bf(bf2f(vf[ct][j]) * w0[j]);
          vw[ks][ct][4 + j] = f2bf(bf2f(vf[ct][4 + j]) * w1[j]);
        }
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        wf[ks][j] = f2bf(w0[j]);
        wf[ks][4 + j] = f2bf(w1[j]);
      }
#pragma unroll
      for (int tt = 2 * ks; tt < 4; ++tt) {
        const bf16x8 pf = load_bf16x8(mb + L::p + (16 * tt + col) * L::PROW + 32 * ks + 8 * g);
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) o[ct][tt] = mfma16(vf[ct], pf, o[ct][tt]);
      }
    }
#pragma unroll
    for (int t = 0; t < 2 * KS; ++t) {
      bf16x8 kf[2];
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const bf16_t* k = mb + L::k + tr_k + 32 * ks * L::KROW + 16 * t;
        kf[ks] = mem_join(mem_read_tr16(k), mem_read_tr16(k + 16 * L::KROW));
      }
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        st[t][ct] *= gamma;
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) st[t][ct] = mfma16(kf[ks], vw[ks][ct], st[t][ct]);
      }
      if constexpr (GATED) {
        if (t % NW == w) {  // every column of the product is the sum of the weighted keys
          f32x4 x = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int ks = 0; ks < 2; ++ks) x = mfma16(kf[ks], wf[ks], x);
          if (col == 0) {
            f32x4* np = reinterpret_cast<f32x4*>(fl + L::n + 16 * t + 4 * g);
            *np = *np * gamma + x;
          }
        }
      }
    }
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) o[ct][tt] *= inv[tt];
    float r[4];
    if (a.slices == 1) {
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        float ss = 0.f;
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
#pragma unroll
          for (int j = 0; j < 4; ++j) ss += o[ct][tt][j] * o[ct][tt][j];
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        if (g == 0) fl[L::ss + w * kMC + 16 * tt + col] = ss;
      }
    }
    __syncthreads();
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) {
      float ss = 0.f;
      if (a.slices == 1) {
#pragma unroll
        for (int i = 0; i < NW; ++i) ss += fl[L::ss + i * kMC + 16 * tt + col];
      }
      r[tt] = 1.f / sqrtf(ss / (float)a.vdim + a.eps);
    }
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) {
      const int t = 16 * tt + col;
      if (t >= nt) continue;
      bf16_t* op = out + (int64_t)(row0 + t0 + t) * a.ldo;
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        const int x = cw + 16 * ct + 4 * g;
        if (x >= a.vdim) continue;
        bf16x4 y;
#pragma unroll
        for (int j = 0; j < 4; ++j)
          y[j] = f2bf(a.slices > 1 ? o[ct][tt][j]
                                   : o[ct][tt][j] * r[tt] * nw[ct][j] *
                                         mem_gate<bf16_t>(bf2f(gate[ct][tt][j]), a.silu));
        *reinterpret_cast<bf16x4*>(op + x) = y;
      }
    }
  }
#pragma unroll
  for (int t = 0; t < 2 * KS; ++t)
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = 16 * t + 4 * g + r, x = cw + 16 * ct + col;
        if (d < a.dim && x < a.vdim) S[(int64_t)d * a.vdim + x] = st[t][ct][r];
      }
  if constexpr (GATED) {
    for (int d = tid; d < a.dim; d += NTHR) N[d] = fl[L::n + d];
    if (tid == 0) top[0] = m0 * (1.f / kLog2e);
  }
}

// ------------------------------------------------------------------ decode
// V columns to a thread, rows spread over the threads that share them; the first rows' loads are in
// flight while queries and keys are prepared.
template <class T, int V>
__global__ __launch_bounds__(256) void memory_decode_kernel(MemoryArgs a) {
  constexpr int U = 16;
  __shared__ float ks[256], qs[256], part[256 * V], os[1024], red[16];
  const int row = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int slot = a.row_state[row];
  T* out = (T*)a.out + (int64_t)row * a.ldo + h * a.vdim;
  if (slot < 0) {
    for (int i = tid; i < a.vdim; i += 256) out[i] = from_f32<T>(0.f);
    return;
  }
  const int pos = a.positions[row];
  const bool gated = a.log_decay == nullptr;
  const T* pr = (const T*)a.proj + (int64_t)row * a.ldp;
  float* S = a.state + ((int64_t)slot * a.H + h) * a.dim * a.vdim;
  const int cg = (a.vdim + V - 1) / V, nc = min(cg, 256), RG = 256 / nc;
  const int rg = tid / nc, c = tid - rg * nc;
  const bool live = rg < RG;
  float s[U][V];
  auto load = [&](int r0, int x) {
#pragma unroll
    for (int i = 0; i < U; ++i) {
      const int r = r0 + i * RG;
#pragma unroll
      for (int v = 0; v < V; ++v) s[i][v] = 0.f;
      if (live && pos > 0 && r < a.dim && x < a.vdim) {
        const float* p = S + (int64_t)r * a.vdim + x;
        if constexpr (V == 4) {
          const f32x4 y = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
          for (int v = 0; v < 4; ++v) s[i][v] = y[v];
        } else {
          s[i][0] = *p;
        }
      }
    }
  };
  load(rg, c * V);
  const int64_t head = (int64_t)slot * a.H + h;
  float nv = 0.f, m = 0.f, f, i;
  if (gated && pos > 0) {
    m = a.top[head * a.slices];
    if (tid < a.dim) nv = a.nrm[head * a.slices * a.dim + tid];
  }
  mem_gates(a, pr, h, f, i);
  const float mn = fmaxf(f + m, i), da = expf(f + m - mn), db = expf(i - mn);
  const float* cs = a.rot_dims ? a.cos_sin + (int64_t)pos * a.rot_dims : nullptr;
  float nq = 0.f;
  if (tid < a.dim) {
    const float q = mem_turned(pr + h * a.dim, tid, cs, a.rot_dims, a.q_scale);
    const float k = mem_turned(pr + a.off_k + h * a.dim, tid, cs, a.rot_dims, a.k_scale);
    qs[tid] = q;
    ks[tid] = k;
    nv = da * nv + db * k;
    nq = nv * q;
    if (gated)
      for (int j = 0; j < a.slices; ++j) a.nrm[(head * a.slices + j) * a.dim + tid] = nv;
  }
  float inv = 1.f;
  if (gated) {
    // the maximum was read by every thread ahead of the barriers of the sum
    inv = 1.f / (fmaxf(fabsf(block_sum(nq, red)), expf(-mn)) + 1e-6f);
    if (tid < a.slices) a.top[head * a.slices + tid] = mn;
  }
  __syncthreads();
  for (int cb = 0; cb < cg; cb += nc) {
    const int x = (cb + c) * V;
    float u[V], o[V];
#pragma unroll
    for (int v = 0; v < V; ++v) {
      o[v] = 0.f;
      u[v] = x + v < a.vdim ? db * to_f32(pr[a.off_v + h * a.vdim + x + v]) : 0.f;
    }
    for (int r0 = rg; r0 < a.dim; r0 += RG * U) {
      if (cb > 0 || r0 > rg) load(r0, x);
#pragma unroll
      for (int j = 0; j < U; ++j) {
        const int r = r0 + j * RG;
        if (r >= a.dim || !live || x >= a.vdim) continue;
        const float k = ks[r], q = qs[r];
        float* p = S + (int64_t)r * a.vdim + x;
        f32x4 y;
#pragma unroll
        for (int v = 0; v < V; ++v) {
          const float z = s[j][v] * da + k * u[v];
          y[v] = z;
          o[v] += q * z;
        }
        if constexpr (V == 4) *reinterpret_cast<f32x4*>(p) = y;
        else *p = y[0];
      }
    }
    if (live) {
#pragma unroll
      for (int v = 0; v < V; ++v) part[tid * V + v] = o[v];
    }
    __syncthreads();
    for (int y = tid; y < nc * V; y += 256) {
      float t = 0.f;
      for (int j = 0; j < RG; ++j) t += part[j * nc * V + y];
      if (cb * V + y < a.vdim) os[cb * V + y] = t * inv;
    }
    __syncthreads();
  }
  float so = 0.f;
  for (int x = tid; x < a.vdim; x += 256) so += os[x] * os[x];
  const float r = 1.f / sqrtf(block_sum(so, red) / (float)a.vdim + a.eps);
  for (int x = tid; x < a.vdim; x += 256)
    out[x] = from_f32<T>(os[x] * r * (a.norm_w ? a.norm_w[h * a.vdim + x] : 1.f) *
                         mem_gate<T>(to_f32(pr[a.off_g + h * a.vdim + x]), a.silu));
}

// Norm and gate of read-outs that several workgroups left in `out`: one (portion, head) each.
template <class T>
__global__ __launch_bounds__(256) void memory_finish_kernel(MemoryArgs a) {
  __shared__ float red[16];
  const int h = blockIdx.y, n = a.seg_len[blockIdx.x], row0 = a.seg_row[blockIdx.x];
  if (a.seg_state[blockIdx.x] < 0) return;
  for (int t = blockIdx.z; t < n; t += gridDim.z) {
    T* o = (T*)a.out + (int64_t)(row0 + t) * a.ldo + h * a.vdim;
    const T* g = (const T*)a.proj + (int64_t)(row0 + t) * a.ldp + a.off_g + h * a.vdim;
    float so = 0.f;
    for (int x = threadIdx.x; x < a.vdim; x += 256) so += to_f32(o[x]) * to_f32(o[x]);
    const float r = 1.f / sqrtf(block_sum(so, red) / (float)a.vdim + a.eps);
    for (int x = threadIdx.x; x < a.vdim; x += 256)
      o[x] = from_f32<T>(to_f32(o[x]) * r * (a.norm_w ? a.norm_w[h * a.vdim + x] : 1.f) *
                         mem_gate<T>(to_f32(g[x]), a.silu));
  }
}

// ------------------------------------------------------------------ launchers
template <class T, int DPL>
static int mem_scan_go(const MemoryArgs& a, hipStream_t st) {
  using S = MemShape<DPL>;
  constexpr int CPL = 4;
  const int cols = a.slices > 1 ? 128 : a.vdim, cp = (cols + 3) & ~3;
  const int groups = (cols + CPL - 1) / CPL + (a.log_decay ? 0 : 1);
  const size_t lds = sizeof(float) * (size_t)(S::CT * (2 * S::DP + 2 * cp + 4));
  memory_scan_kernel<T, DPL, CPL>
      <<<dim3(a.nseg, a.H, a.slices), dim3((groups * 8 + 63) / 64 * 64), lds, st>>>(a);
  return 0;
}
template <class T>
static int mem_scan_t(const MemoryArgs& a, hipStream_t st) {
  if (a.dim <= 32) return mem_scan_go<T, 4>(a, st);
  if (a.dim <= 64) return mem_scan_go<T, 8>(a, st);
  if (a.dim <= 128) return mem_scan_go<T, 16>(a, st);
  return mem_scan_go<T, 32>(a, st);
}

template <int KS, int NW, int CT>
static int mem_chunk_go(const MemoryArgs& a, hipStream_t st) {
  using L = MemLds<KS, NW, CT>;
  const dim3 grid(a.nseg, a.H, a.slices), blk(64 * NW);
  if (a.log_decay) memory_chunk_kernel<KS, NW, CT, false><<<grid, blk, L::BYTES, st>>>(a);
  else memory_chunk_kernel<KS, NW, CT, true><<<grid, blk, L::BYTES, st>>>(a);
  return 0;
}
template <int KS>
static int mem_chunk_c(const MemoryArgs& a, hipStream_t st) {
  constexpr bool wide = KS == 8;  // 8 waves of one column tile: as many accumulators to a wave
  if (a.slices == 1 && a.vdim > 128) return mem_chunk_go<KS, 8, 2>(a, st);
  if (a.slices == 1 && a.vdim <= 64) return mem_chunk_go<KS, 4, 1>(a, st);
  return mem_chunk_go<KS, wide ? 8 : 4, wide ? 1 : 2>(a, st);
}

static int mem_check(const MemoryArgs& a) {
  if (a.H < 1 || a.dim < 1 || a.dim > 256 || a.vdim < 1 || a.vdim > 1024) return -1;
  if (a.slices != (a.vdim <= 256 ? 1 : (a.vdim + 127) / 128)) return -1;
  if (a.rot_dims < 0 || a.rot_dims % 2 || a.rot_dims > a.dim || (a.rot_dims && !a.cos_sin)) return -1;
  if (!a.log_decay && (!a.i_bias || !a.f_bias || !a.nrm || !a.top || !(a.cap > 0.f))) return -1;
  return 0;
}

// plain: token by token also where the chunk form takes the sizes
int launch_memory_scan(int f32, const MemoryArgs& a, int plain, hipStream_t st) {
  if (a.nseg == 0) return 0;
  if (mem_check(a)) return -1;
  const bool chunk = !f32 && !plain && a.dim % 16 == 0 && a.rot_dims % 16 == 0 && a.vdim % 8 == 0 &&
                     a.ldp % 8 == 0 && a.off_k % 8 == 0 && a.off_v % 8 == 0 && a.off_g % 4 == 0 &&
                     a.ldo % 4 == 0;
  int rc;
  if (chunk) {
    if (a.dim <= 32) rc = mem_chunk_c<1>(a, st);
    else if (a.dim <= 64) rc = mem_chunk_c<2>(a, st);
    else if (a.dim <= 128) rc = mem_chunk_c<4>(a, st);
    else rc = mem_chunk_c<8>(a, st);
  } else {
    rc = f32 ? mem_scan_t<float>(a, st) : mem_scan_t<bf16_t>(a, st);
  }
  if (rc) return rc;
  if (a.slices > 1) {
    const dim3 grid(a.nseg, a.H, std::min(64, std::max(1, a.rows / a.nseg)));
    if (f32) memory_finish_kernel<float><<<grid, dim3(256), 0, st>>>(a);
    else memory_finish_kernel<bf16_t><<<grid, dim3(256), 0, st>>>(a);
  }
  return (int)hipGetLastError();
}

int launch_memory_decode(int f32, const MemoryArgs& a, hipStream_t st) {
  if (a.rows == 0) return 0;
  if (mem_check(a)) return -1;
  const dim3 grid(a.rows, a.H), blk(256);
  const bool vec = a.vdim % 4 == 0;
  if (f32) {
    if (vec) memory_decode_kernel<float, 4><<<grid, blk, 0, st>>>(a);
    else memory_decode_kernel<float, 1><<<grid, blk, 0, st>>>(a);
  } else {
    if (vec) memory_decode_kernel<bf16_t, 4><<<grid, blk, 0, st>>>(a);
    else memory_decode_kernel<bf16_t, 1><<<grid, blk, 0, st>>>(a);
  }
  return (int)hipGetLastError();
}

// dynamic LDS above 64 KB
template <int KS, int NW, int CT>
static int mem_attr() {
  const int n = (int)MemLds<KS, NW, CT>::BYTES;
  static_assert(MemLds<KS, NW, CT>::BYTES <= 160 * 1024, "LDS of a CU");
  return (int)hipFuncSetAttribute((const void*)memory_chunk_kernel<KS, NW, CT, true>,
                                  hipFuncAttributeMaxDynamicSharedMemorySize, n) |
         (int)hipFuncSetAttribute((const void*)memory_chunk_kernel<KS, NW, CT, false>,
                                  hipFuncAttributeMaxDynamicSharedMemorySize, n);
}
template <int KS>
static int mem_attrs() {
  return mem_attr<KS, 8, 2>() | mem_attr<KS, 4, 1>() |
         mem_attr<KS, KS == 8 ? 8 : 4, KS == 8 ? 1 : 2>();
}
int configure_memory() {
  return mem_attrs<1>() | mem_attrs<2>() | mem_attrs<4>() | mem_attrs<8>();
}

}  // namespace drtc
