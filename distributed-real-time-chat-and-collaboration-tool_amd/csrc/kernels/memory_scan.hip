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
      const float f = t < nt ? av[t] : 0.f, i = t < nt ? bv[t] : kNegBig, mn = fmaxf(f + mm, i);
      da[t] = expf(f + mm - mn);
      db[t] = expf(i - mn);
      mm = mn;
      if (tid == 0) em[t] = expf(-mn);
    }
    m = mm;
    if (live) {
#pragma unroll
      for (int t = 0; t < CT; ++t) {
        if (t >= nt) continue;
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
// weights of the update go onto the V fragments in registers.  The scales of queries and keys ride
// on the exponents and weights, so unrotated rows are staged as they are.
constexpr int kMC = 64;

typedef short mem_s16x4 __attribute__((ext_vector_type(4)));
typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));
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
// 16 / 8 bytes at a 32-bit byte offset from a base all lanes share
DRTC_DEVICE bf16x8 mem_at8(const bf16_t* base, unsigned off) {
  return *reinterpret_cast<const bf16x8*>(reinterpret_cast<const char*>(base) + off);
}
DRTC_DEVICE bf16x4 mem_at4(const bf16_t* base, unsigned off) {
  return *reinterpret_cast<const bf16x4*>(reinterpret_cast<const char*>(base) + off);
}
// v of another lane by DPP; lanes without a source: `other`
template <int CTRL, int ROWS>
DRTC_DEVICE float lane_from(float v, float other) {
  return __int_as_float(__builtin_amdgcn_update_dpp(__float_as_int(other), __float_as_int(v), CTRL,
                                                    ROWS, 0xF, false));
}
// Inclusive scan over the lanes of a wave: within rows of 16, then the rows' last lanes on.
template <class Op>
DRTC_DEVICE float lane_scan(float v, float zero, Op op) {
  v = op(v, lane_from<0x111, 0xF>(v, zero));
  v = op(v, lane_from<0x112, 0xF>(v, zero));
  v = op(v, lane_from<0x114, 0xF>(v, zero));
  v = op(v, lane_from<0x118, 0xF>(v, zero));
  v = op(v, lane_from<0x142, 0xA>(v, zero));
  return op(v, lane_from<0x143, 0xC>(v, zero));
}
DRTC_DEVICE float last_lane(float v) {
  return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), 63));
}
// cap tanh(x / cap) and log2 sigmoid by hardware exp2 / log2; for large x the latter's series, where
// 1 + e^-x would round
DRTC_DEVICE float cap_hw(float x, float cap, float inv) {
  return cap - 2.f * cap * __builtin_amdgcn_rcpf(1.f + fast_exp2(x * inv * (2.f * kLog2e)));
}
DRTC_DEVICE float logsig2_hw(float x) {
  const float e = fast_exp2(-x * kLog2e);
  const float l = __builtin_amdgcn_logf(1.f + e), y = e * (1.f - e * (0.5f - e * (1.f / 3.f))) * kLog2e;
  return x < -30.f ? x * kLog2e : x > 6.f ? -y : -l;
}

// KS: 32-dim steps of a key (padded); NW waves of 16 columns
template <int KS, int NW>
struct MemLds {
  static constexpr int DP = 32 * KS, COLS = 16 * NW, NG = NW / 4;
  static constexpr int QROW = DP + 8, KROW = DP + 16, VROW = COLS + 16, PROW = kMC + 8;
  // bf16 elements, then floats
  static constexpr int q = 0, k = q + kMC * QROW, v = k + kMC * KROW, p = v + kMC * VROW;
  static constexpr int bf = p + kMC * PROW;
  // gates of two chunks: g, M, 2^(m_0 - M), 2^-m, update weights, the state's factor
  static constexpr int G = 5 * kMC + 4, m = kMC, in = 2 * kMC, em = 3 * kMC, w = 4 * kMC, ga = 5 * kMC;
  static constexpr int n = 2 * G, qn = n + 2 * DP, rs = qn + kMC, ss = rs + NG * kMC, fl = ss + NW * kMC;  // ss [token][wave]
  static constexpr size_t BYTES = (size_t)bf * 2 + (size_t)fl * 4;
};

template <int KS, int NW, bool GATED, bool ROT>
__global__ __launch_bounds__(64 * NW, 2) void memory_chunk_kernel(MemoryArgs a) {
  using L = MemLds<KS, NW>;
  constexpr int NTHR = 64 * NW, PU = L::DP / 16, NU = (kMC * PU + NTHR - 1) / NTHR, NV = 2;
  extern __shared__ __attribute__((aligned(16))) bf16_t mb[];
  float* fl = reinterpret_cast<float*>(mb + L::bf);
  const int seg = blockIdx.x, h = blockIdx.y, sl = blockIdx.z, c0 = sl * L::COLS;
  const int slot = a.seg_state[seg];
  const int n = a.seg_len[seg], row0 = a.seg_row[seg], pos0 = a.seg_pos[seg];
  const int tid = threadIdx.x, w = wave_id_uniform(), lane = tid & 63, col = lane & 15, g = lane >> 4;
  const int cols = min(L::COLS, a.vdim - c0);
  bf16_t* out = (bf16_t*)a.out + (int64_t)row0 * a.ldo + h * a.vdim + c0;
  if (slot < 0) {
    for (int i = tid; i < n * cols; i += NTHR) out[(int64_t)(i / cols) * a.ldo + i % cols] = f2bf(0.f);
    return;
  }
  const bf16_t* proj = (const bf16_t*)a.proj + (int64_t)row0 * a.ldp;
  const int cw = 16 * w;  // this wave's first column of the workgroup's
  const bool own = cw < cols;
  const int nwave = (cols - 1) >> 4;  // keeps the normaliser
  float* S = a.state + ((int64_t)slot * a.H + h) * a.dim * a.vdim + c0;
  float* N = GATED ? a.nrm + (((int64_t)slot * a.H + h) * a.slices + sl) * a.dim : nullptr;
  float* top = GATED ? a.top + ((int64_t)slot * a.H + h) * a.slices + sl : nullptr;

  f32x4 st[2 * KS];
#pragma unroll
  for (int t = 0; t < 2 * KS; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * t + 4 * g + r, x = cw + col;
      st[t][r] = pos0 > 0 && d < a.dim && x < cols ? S[d * a.vdim + x] : 0.f;
    }
  if constexpr (GATED) {
    for (int d = tid; d < L::DP; d += NTHR) fl[L::n + d] = pos0 > 0 && d < a.dim ? N[d] : 0.f;
  }

  // staging: a unit is two 8-element vectors of a token's query and key - the two halves of eight
  // rotated pairs, or neighbours behind the rotated part.  Tokens behind the portion repeat its
  // last one: their weights are zero.
  const int half = a.rot_dims >> 1;
  int tok[NU], e0[NU], e1[NU];
  bool in_u[NU], turn[NU];
#pragma unroll
  for (int i = 0; i < NU; ++i) {
    const int u = tid + i * NTHR, pr = u % PU;
    in_u[i] = u < kMC * PU && 16 * pr < a.dim;
    tok[i] = in_u[i] ? u / PU : 0;
    turn[i] = ROT && in_u[i] && 16 * pr < a.rot_dims;
    e0[i] = !in_u[i] ? 0 : turn[i] ? 8 * pr : 16 * pr;
    e1[i] = turn[i] ? e0[i] + half : e0[i] + 8;
  }
  bf16x8 pq[NU][2], pk[NU][2], pv[NV];
  float cs[ROT ? NU : 1][2][8];
  // without branches, so that no wait for one load becomes a wait for all
  auto prefetch = [&](int t0) {
    const bf16_t *qb = proj + (int64_t)t0 * a.ldp + h * a.dim, *kb = qb + a.off_k;
    const float* cb = a.cos_sin + (int64_t)(pos0 + t0) * a.rot_dims;
    const int last = n - 1 - t0;
#pragma unroll
    for (int i = 0; i < NU; ++i) {
      const unsigned tk = min(tok[i], last), r = tk * a.ldp;
      const unsigned o0 = 2 * (r + e0[i]), o1 = 2 * (r + e1[i]);
      pq[i][0] = mem_at8(qb, o0);
      pq[i][1] = mem_at8(qb, o1);
      pk[i][0] = mem_at8(kb, o0);
      pk[i][1] = mem_at8(kb, o1);
      if constexpr (ROT) {
        const unsigned c = tk * a.rot_dims + (turn[i] ? e0[i] : 0);
        load8(cs[i][0], cb + c);
        load8(cs[i][1], cb + c + half);
      }
    }
    const bf16_t* vb = proj + (int64_t)t0 * a.ldp + a.off_v + h * a.vdim + c0;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = tid + i * NTHR, tk = v / (L::COLS / 8), c = (v % (L::COLS / 8)) * 8;
      pv[i] = mem_at8(vb, 2u * (unsigned)(min(tk, last) * a.ldp + min(c, cols - 8)));
    }
  };
  prefetch(0);
  {  // columns behind the head and the values stay zero
    bf16x8 z;
#pragma unroll
    for (int j = 0; j < 8; ++j) z[j] = f2bf(0.f);
    const int dv = L::DP / 8, lo = a.dim / 8;
    for (int i = tid; i < kMC * (dv - lo); i += NTHR) {
      const int t = i / (dv - lo), c = (lo + i % (dv - lo)) * 8;
      store_bf16x8(mb + L::q + t * L::QROW + c, z);
      store_bf16x8(mb + L::k + t * L::KROW + c, z);
    }
    const int vv = L::COLS / 8, vlo = cols / 8;
    for (int i = tid; i < kMC * (vv - vlo); i += NTHR)
      store_bf16x8(mb + L::v + (i / (vv - vlo)) * L::VROW + (vlo + i % (vv - vlo)) * 8, z);
  }

  // gates of a chunk, one token to a lane of the first wave, a chunk ahead of their use
  float m0 = 0.f;  // log2 units
  bf16_t gi = f2bf(0.f), gf = f2bf(0.f);
  const float f2 = GATED ? 0.f : a.log_decay[h] * kLog2e;
  const float lk = log2f(a.k_scale), lq = log2f(a.q_scale), inv_cap = GATED ? 1.f / a.cap : 0.f;
  const float ib = GATED ? a.i_bias[h] : 0.f, fb = GATED ? a.f_bias[h] : 0.f;
  auto load_gates = [&](int t0) {
    if constexpr (GATED) {
      const bf16_t* r = proj + (int64_t)min(t0 + lane, n - 1) * a.ldp + h;
      gi = r[a.off_i];
      gf = r[a.off_f];
    }
  };
  auto gates = [&](int t0, float* b) {
    const int nt = min(kMC, n - t0);
    float F, gg, M;
    if constexpr (GATED) {
      const float f = logsig2_hw(cap_hw(bf2f(gf) + fb, a.cap, inv_cap));
      F = lane_scan(lane < nt ? f : 0.f, 0.f, [](float x, float y) { return x + y; });
      gg = lane < nt ? cap_hw(bf2f(gi) + ib, a.cap, inv_cap) * kLog2e - F : kNegBig;
      M = fmaxf(m0, lane_scan(gg, kNegBig, [](float x, float y) { return fmaxf(x, y); }));
    } else {
      F = (float)min(lane + 1, nt) * f2;
      gg = -F;
      M = -F;
    }
    const float M1 = last_lane(M);
    b[lane] = gg + lk;
    b[L::m + lane] = M - lq;
    b[L::in + lane] = fast_exp2(m0 - M) * a.q_scale;
    b[L::em + lane] = fast_exp2(-(F + M));
    b[L::w + lane] = lane < nt ? fast_exp2(gg - M1) * a.k_scale : 0.f;
    if (lane == 0) b[L::ga] = fast_exp2(m0 - M1);
    if constexpr (GATED) m0 = last_lane(F) + M1;
  };
  if (w == 0) {
    if (GATED && pos0 > 0) m0 = top[0] * kLog2e;
    load_gates(0);
    gates(0, fl);
    load_gates(kMC);
  }
  const int tr_k = ((col >> 2) + 4 * g) * L::KROW + 4 * (col & 3);
  const int tr_v = ((col >> 2) + 4 * g) * L::VROW + 4 * (col & 3) + cw;
  f32x4 nw;
#pragma unroll
  for (int r = 0; r < 4; ++r)
    nw[r] = a.norm_w && cw + 4 * g + r < cols ? a.norm_w[h * a.vdim + c0 + cw + 4 * g + r] : 1.f;
  const float inv_dv = 1.f / (float)a.vdim;

  float* cur = fl;
  for (int t0 = 0; t0 < n; t0 += kMC) {
    float* nxt = cur == fl ? fl + L::G : fl;
    const float* nc = fl + L::n + (cur == fl ? 0 : L::DP);  // the normaliser, and after this chunk
    float* nn = fl + L::n + (cur == fl ? L::DP : 0);
    const int nt = min(kMC, n - t0);
    bf16x4 gate[4];  // read-out gates of this chunk
    {
      const bf16_t* base = proj + (int64_t)t0 * a.ldp + a.off_g + h * a.vdim + c0;
      const int x = min(cw + 4 * g, cols - 4);
#pragma unroll
      for (int tt = 0; tt < 4; ++tt)
        gate[tt] = mem_at4(base, 2u * (unsigned)(min(16 * tt + col, nt - 1) * a.ldp + x));
    }
#pragma unroll
    for (int i = 0; i < NU; ++i) {
      if constexpr (ROT) {
        if (turn[i]) {
          auto rotate = [&](bf16x8 (&x)[2]) {
#pragma unroll
            for (int j = 0; j < 8; ++j) {
              const float c = cs[i][0][j], s = cs[i][1][j], x0 = bf2f(x[0][j]), x1 = bf2f(x[1][j]);
              x[0][j] = f2bf(x0 * c - x1 * s);
              x[1][j] = f2bf(x1 * c + x0 * s);
            }
          };
          rotate(pq[i]);
          rotate(pk[i]);
        }
      }
      if (in_u[i]) {
        bf16_t *qd = mb + L::q + tok[i] * L::QROW, *kd = mb + L::k + tok[i] * L::KROW;
        store_bf16x8(qd + e0[i], pq[i][0]);
        store_bf16x8(qd + e1[i], pq[i][1]);
        store_bf16x8(kd + e0[i], pk[i][0]);
        store_bf16x8(kd + e1[i], pk[i][1]);
      }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = tid + i * NTHR, c = (v % (L::COLS / 8)) * 8;
      if (c < cols) store_bf16x8(mb + L::v + (v / (L::COLS / 8)) * L::VROW + c, pv[i]);
    }
    prefetch(min(t0 + kMC, n - 1));
    __syncthreads();

    // what does not need the scores of other waves: the weighted scores of 16 tokens to a wave (8
    // waves: every other key tile), the read-out of the state, its update
    {
      const int tt = w & 3, t = 16 * tt + col;
      const float Mt = cur[L::m + t];
      bf16x8 qf[KS];
#pragma unroll
      for (int s = 0; s < KS; ++s) qf[s] = load_bf16x8(mb + L::q + t * L::QROW + 32 * s + 8 * g);
      float rsum = 0.f;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt) {
        if (kt % L::NG != (w >> 2) || kt > (tt | 1)) continue;
        bf16x4 pf;
#pragma unroll
        for (int r = 0; r < 4; ++r) pf[r] = f2bf(0.f);
        if (kt <= tt) {
          f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int s = 0; s < KS; ++s)
            sc = mfma16(load_bf16x8(mb + L::k + (16 * kt + col) * L::KROW + 32 * s + 8 * g), qf[s], sc);
          const f32x4 gj = *reinterpret_cast<const f32x4*>(cur + 16 * kt + 4 * g);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float p = 16 * kt + 4 * g + r <= t ? sc[r] * fast_exp2(gj[r] - Mt) : 0.f;
            rsum += p;
            pf[r] = f2bf(p);
          }
        }
        // keys in the order of the V fragments: 4 g + r of both tiles of a 32-key step together
        *reinterpret_cast<bf16x4*>(mb + L::p + t * L::PROW + 32 * (kt >> 1) + 8 * g + 4 * (kt & 1)) = pf;
      }
      if constexpr (GATED) {
        rsum += __shfl_xor(rsum, 16, 64);
        rsum += __shfl_xor(rsum, 32, 64);
        if (g == 0) fl[L::rs + (w >> 2) * kMC + t] = rsum;
        constexpr int PART = L::DP / NW;  // n.q: NW lanes to a token
        const int tk = tid / NW, part = tid % NW;
        float d = 0.f;
#pragma unroll
        for (int j = 0; j < PART; j += 4) {
          const bf16x4 q4 = load_bf16x4(mb + L::q + tk * L::QROW + part * PART + j);
          const f32x4 n4 = *reinterpret_cast<const f32x4*>(nc + part * PART + j);
#pragma unroll
          for (int r = 0; r < 4; ++r) d += bf2f(q4[r]) * n4[r];
        }
        d = NW == 4 ? quad_sum(d) : sum8(d);
        if (part == 0) fl[L::qn + tk] = d;
      }
      if (w == 0 && t0 + kMC < n) {
        gates(t0 + kMC, nxt);
        load_gates(t0 + 2 * kMC);
      }
    }
    f32x4 o[4];
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) o[tt] = (f32x4){0.f, 0.f, 0.f, 0.f};
    bf16x8 vf[2];
    if (own) {
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        bf16x8 hi, lo;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float x = st[2 * s + (j >> 2)][j & 3];
          hi[j] = f2bf(x);
          lo[j] = f2bf(x - bf2f(hi[j]));
        }
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
          const bf16_t* q = mb + L::q + (16 * tt + col) * L::QROW + 32 * s + 4 * g;
          const bf16x8 qf = mem_join(load_bf16x4(q), load_bf16x4(q + 16));
          o[tt] = mfma16(hi, qf, o[tt]);
          o[tt] = mfma16(lo, qf, o[tt]);
        }
      }
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) o[tt] *= cur[L::in + 16 * tt + col];
      bf16x8 vw[2], wf[2];
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const f32x4 w0 = *reinterpret_cast<const f32x4*>(cur + L::w + 32 * ks + 4 * g);
        const f32x4 w1 = *reinterpret_cast<const f32x4*>(cur + L::w + 32 * ks + 16 + 4 * g);
        const bf16_t* v = mb + L::v + tr_v + 32 * ks * L::VROW;
        vf[ks] = mem_join(mem_read_tr16(v), mem_read_tr16(v + 16 * L::VROW));
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          vw[ks][j] = f2bf(bf2f(vf[ks][j]) * w0[j]);
          vw[ks][4 + j] = f2bf(bf2f(vf[ks][4 + j]) * w1[j]);
          if constexpr (GATED) {
            wf[ks][j] = f2bf(w0[j]);
            wf[ks][4 + j] = f2bf(w1[j]);
          }
        }
      }
      const float gamma = cur[L::ga];
#pragma unroll
      for (int t = 0; t < 2 * KS; ++t) {
        st[t] *= gamma;
        f32x4 x = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
          const bf16_t* k = mb + L::k + tr_k + 32 * ks * L::KROW + 16 * t;
          const bf16x8 kf = mem_join(mem_read_tr16(k), mem_read_tr16(k + 16 * L::KROW));
          st[t] = mfma16(kf, vw[ks], st[t]);
          // the normaliser, by the last wave: every column of the product is the sum of the
          // weighted keys
          if constexpr (GATED) {
            if (w == nwave) x = mfma16(kf, wf[ks], x);
          }
        }
        if constexpr (GATED) {
          if (w == nwave && col == 0) {
            const int d = 16 * t + 4 * g;
            *reinterpret_cast<f32x4*>(nn + d) = *reinterpret_cast<const f32x4*>(nc + d) * gamma + x;
          }
        }
      }
    }
    __syncthreads();

    if (own) {
#pragma unroll
      for (int ks = 0; ks < 2; ++ks)
#pragma unroll
        for (int tt = 2 * ks; tt < 4; ++tt)
          o[tt] = mfma16(vf[ks], load_bf16x8(mb + L::p + (16 * tt + col) * L::PROW + 32 * ks + 8 * g), o[tt]);
      if constexpr (GATED) {
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) {
          const int t = 16 * tt + col;
          float d = cur[L::in + t] * fl[L::qn + t];
#pragma unroll
          for (int i = 0; i < L::NG; ++i) d += fl[L::rs + i * kMC + t];
          o[tt] *= __builtin_amdgcn_rcpf(fmaxf(fabsf(d), cur[L::em + t]) + 1e-6f);
        }
      }
    }
    if (a.slices == 1) {
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
        float ss = 0.f;
        if (own) {
#pragma unroll
          for (int j = 0; j < 4; ++j) ss += o[tt][j] * o[tt][j];
        }
        ss += __shfl_xor(ss, 16, 64);
        ss += __shfl_xor(ss, 32, 64);
        if (g == 0) fl[L::ss + (16 * tt + col) * NW + w] = ss;
      }
    }
    __syncthreads();
    // stores without branches (rows behind the portion and columns behind the head are beyond the
    // buffer's end), so that the next wait for loads does not wait for them
    const __amdgpu_buffer_rsrc_t ob = __builtin_amdgcn_make_buffer_rsrc(
        (void*)(out + (int64_t)t0 * a.ldo), (short)0, 2 * nt * a.ldo, 0x00020000);
#pragma unroll
    for (int tt = 0; tt < 4; ++tt) {
      const int t = 16 * tt + col;
      if (a.slices == 1) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NW; i += 4) {
          const f32x4 x = *reinterpret_cast<const f32x4*>(fl + L::ss + t * NW + i);
          ss += (x[0] + x[1]) + (x[2] + x[3]);
        }
        o[tt] *= __builtin_amdgcn_rsqf(ss * inv_dv + a.eps);
        if (a.norm_w) o[tt] *= nw;
#pragma unroll
        for (int j = 0; j < 4; ++j) o[tt][j] *= mem_gate<bf16_t>(bf2f(gate[tt][j]), a.silu);
      }
      bf16x4 y;
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = f2bf(o[tt][j]);
      __builtin_amdgcn_raw_buffer_store_b64(
          __builtin_bit_cast(u32x2, y), ob,
          cw + 4 * g < cols ? 2u * (unsigned)(t * a.ldo + cw + 4 * g) : 0xFFFFFFF0u, 0, 0);
    }
    cur = nxt;
  }
  int gl = g;  // addresses of the state are computed again rather than kept through the loop
  asm volatile("" : "+v"(gl));
#pragma unroll
  for (int t = 0; t < 2 * KS; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * t + 4 * gl + r, x = cw + col;
      if (d < a.dim && x < cols) S[d * a.vdim + x] = st[t][r];
    }
  if constexpr (GATED) {
    const float* nc = fl + L::n + (cur == fl ? 0 : L::DP);
    for (int d = tid; d < a.dim; d += NTHR) N[d] = nc[d];
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

template <int KS, int NW>
static int mem_chunk_go(const MemoryArgs& a, hipStream_t st) {
  using L = MemLds<KS, NW>;
  const dim3 grid(a.nseg, a.H, a.slices), blk(64 * NW);
  if (!a.log_decay) memory_chunk_kernel<KS, NW, true, false><<<grid, blk, L::BYTES, st>>>(a);
  else if (a.rot_dims) memory_chunk_kernel<KS, NW, false, true><<<grid, blk, L::BYTES, st>>>(a);
  else memory_chunk_kernel<KS, NW, false, false><<<grid, blk, L::BYTES, st>>>(a);
  return 0;
}
template <int KS>
static int mem_chunk_w(const MemoryArgs& a, hipStream_t st) {
  if (a.slices == 1 && a.vdim <= 64) return mem_chunk_go<KS, 4>(a, st);
  return mem_chunk_go<KS, 8>(a, st);
}

static int mem_check(const MemoryArgs& a) {
  if (a.H < 1 || a.dim < 1 || a.dim > 256 || a.vdim < 1 || a.vdim > 1024) return -1;
  if (a.slices != (a.vdim + 127) / 128) return -1;
  if (a.rot_dims < 0 || a.rot_dims % 2 || a.rot_dims > a.dim || (a.rot_dims && !a.cos_sin)) return -1;
  if (!a.log_decay && a.rot_dims) return -1;
  if (!a.log_decay && (!a.i_bias || !a.f_bias || !a.nrm || !a.top || !(a.cap > 0.f))) return -1;
  return 0;
}

// plain: token by token also where the chunk form takes the sizes
int launch_memory_scan(int f32, const MemoryArgs& a, int plain, hipStream_t st) {
  if (a.nseg == 0) return 0;
  if (mem_check(a)) return -1;
  const bool chunk = !f32 && !plain && a.dim % 16 == 0 && a.rot_dims % 16 == 0 && a.vdim % 8 == 0 &&
                     a.ldp % 8 == 0 && a.off_k % 8 == 0 && a.off_v % 8 == 0 && a.off_g % 4 == 0 &&
                     a.ldo % 4 == 0 && a.ldp < (1 << 23) && a.ldo < (1 << 23);
  int rc;
  if (chunk) {
    if (a.dim <= 32) rc = mem_chunk_w<1>(a, st);
    else if (a.dim <= 64) rc = mem_chunk_w<2>(a, st);
    else if (a.dim <= 128) rc = mem_chunk_w<4>(a, st);
    else rc = mem_chunk_w<8>(a, st);
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
template <int KS, int NW>
static int mem_attr() {
  const int n = (int)MemLds<KS, NW>::BYTES;
  static_assert(MemLds<KS, NW>::BYTES <= 160 * 1024, "LDS of a CU");
  int e = 0;
  for (const void* f : {(const void*)memory_chunk_kernel<KS, NW, true, false>,
                        (const void*)memory_chunk_kernel<KS, NW, false, true>,
                        (const void*)memory_chunk_kernel<KS, NW, false, false>})
    e |= (int)hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, n);
  return e;
}
template <int KS>
static int mem_attrs() {
  return mem_attr<KS, 4>() | mem_attr<KS, 8>();
}
int configure_memory() {
  return mem_attrs<1>() | mem_attrs<2>() | mem_attrs<4>() | mem_attrs<8>();
}

}  // namespace drtc
