// Latent attention (gfx950): per-token key/value latents in a paged cache, a rotated key part
// shared by all heads, sliding window, softmax sinks, sigmoid gates per head.
//
// Cache row of a token (LW elements, a multiple of 32):  [ latent R | rotated key r | 0 ... ]
// 32 rows to a block.  A step runs
//   latent_prep      RMS norm of the latent, rotary on its key part and on the queries, cache
//                    write - one workgroup per token
//   prompt portions  per-head keys / values are projected up from the latents of the portion
//                    and of the window ahead of it (latent_gather + a GEMM), then varlen flash
//                    attention on MFMA (latent_prefill_kernel)
//   decode           the query is projected down into the latent space instead (head_gemm), so
//                    all heads attend to the SAME cached rows, which are both keys (all LW
//                    columns) and values (the first R): latent_decode_kernel stages each
//                    32-token block in LDS once for up to 64 heads; the result goes back up
//                    per head (head_gemm)
// bf16 runs on MFMA with the operand maps of attention_prefill.hip; sizes those do not cover,
// and fp32, run the *_any kernels.
#include "attend_any.h"
#include "hybrid_launchers.h"

#include <algorithm>

namespace drtc {

constexpr int kLB = 32;  // tokens per cache block

typedef short lat_s16x4 __attribute__((ext_vector_type(4)));
DRTC_DEVICE bf16x4 lat_read_tr16(const bf16_t* p) {
  lat_s16x4 v = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) lat_s16x4*)(p));
  return __builtin_bit_cast(bf16x4, v);
}
// Factor of a head's output: 1, or the sigmoid of its gate input.
template <class T>
DRTC_DEVICE float head_gate(const void* gate, int64_t at) {
  return gate ? 1.f / (1.f + expf(-to_f32(((const T*)gate)[at]))) : 1.f;
}
DRTC_DEVICE bf16x8 zero8() {
  bf16x8 z;
#pragma unroll
  for (int j = 0; j < 8; ++j) z[j] = f2bf(0.f);
  return z;
}

// ------------------------------------------------------------------ per-token preparation
// One workgroup per token.  V: elements a thread moves at once (8, or 2 where the sizes or the
// rows do not align); pairs never straddle a vector.
template <class T, int V>
DRTC_DEVICE void lat_load(float (&v)[V], const T* p) {
  if constexpr (V == 8) load8(v, p);
  else {
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = to_f32(p[j]);
  }
}
template <class T, int V>
DRTC_DEVICE void lat_store(T* p, const float (&v)[V]) {
  if constexpr (V == 8) store8(p, v);
  else {
#pragma unroll
    for (int j = 0; j < V; ++j) p[j] = from_f32<T>(v[j]);
  }
}

template <class T, int V>
__global__ __launch_bounds__(256) void latent_prep_kernel(LatentPrepArgs a) {
  __shared__ float red[16];
  const int row = blockIdx.x, tid = threadIdx.x;
  T* pr = (T*)a.proj + (int64_t)row * a.ldp;
  const T* kv = pr + a.off_kv;
  const int half = a.rot_dims >> 1;
  const float* cs = a.cos_sin + (int64_t)a.positions[row] * a.rot_dims;
  // V elements of a rotated part from element i on
  auto turn = [&](const T* src, T* dst, int i) {
    float x[V];
    lat_load<T, V>(x, src + i);
#pragma unroll
    for (int j = 0; j < V; j += 2) {
      const int k = (i + j) >> 1;
      if (k < half) {
        const float u = x[j], v = x[j + 1], c = cs[k], s = cs[half + k];
        x[j] = u * c - v * s;
        x[j + 1] = v * c + u * s;
      }
    }
    lat_store<T, V>(dst + i, x);
  };
  // queries: in place, or into the latent-space query rows
  const int dq = a.dim + a.rot;
  if (a.qa) {
    const int tail = (a.LW - a.R) / V, own = a.rot / V;
    for (int k = tid; k < a.H * tail; k += 256) {
      const int h = k / tail, i = k - h * tail;
      T* d = (T*)a.qa + ((int64_t)row * a.H + h) * a.LW + a.R;
      if (i < own) turn(pr + h * dq + a.dim, d, i * V);
      else {
#pragma unroll
        for (int j = 0; j < V; ++j) d[i * V + j] = from_f32<T>(0.f);
      }
    }
  } else {
    const int per = (a.rot_dims + V - 1) / V;
    for (int k = tid; k < a.H * per; k += 256) {
      const int h = k / per;
      T* q = pr + h * dq + a.dim;
      turn(q, q, (k - h * per) * V);
    }
  }
  if (a.off_kv < 0) return;  // the latents are another layer's
  const int64_t slot = a.slots ? a.slots[row] : -1;
  T* lat = a.lat ? (T*)a.lat + (int64_t)row * a.LW : nullptr;
  T* cache = a.cache && slot >= 0 ? (T*)a.cache + slot * a.LW : nullptr;
  float ss = 0.f;
  for (int i = tid * V; i < a.R; i += 256 * V) {
    float x[V];
    lat_load<T, V>(x, kv + i);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += x[j] * x[j];
  }
  const float rinv = 1.f / sqrtf(block_sum(ss, red) / (float)a.R + a.eps);
  for (int i = tid * V; i < a.LW; i += 256 * V) {
    float x[V];
    if (i < a.R) {
      lat_load<T, V>(x, kv + i);
#pragma unroll
      for (int j = 0; j < V; ++j) x[j] *= rinv * a.norm_w[i + j];
    } else if (i < a.R + a.rot) {
      lat_load<T, V>(x, kv + i);
#pragma unroll
      for (int j = 0; j < V; j += 2) {
        const int k = (i + j - a.R) >> 1;
        if (k < half) {
          const float u = x[j], v = x[j + 1], c = cs[k], s = cs[half + k];
          x[j] = u * c - v * s;
          x[j + 1] = v * c + u * s;
        }
      }
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) x[j] = 0.f;
    }
    if (lat) lat_store<T, V>(lat + i, x);
    if (cache) lat_store<T, V>(cache + i, x);
  }
}

template <class T>
static void lat_prep_t(const LatentPrepArgs& a, hipStream_t st) {
  if (a.R % 8 == 0 && a.rot % 8 == 0 && a.dim % 8 == 0 && a.ldp % 8 == 0 &&
      (a.off_kv < 0 || a.off_kv % 8 == 0) && a.LW % 8 == 0)
    latent_prep_kernel<T, 8><<<dim3(a.rows), dim3(256), 0, st>>>(a);
  else
    latent_prep_kernel<T, 2><<<dim3(a.rows), dim3(256), 0, st>>>(a);
}

int launch_latent_prep(int f32, const LatentPrepArgs& a, hipStream_t st) {
  if (a.rows == 0) return 0;
  if (a.rot_dims > a.rot || a.rot_dims % 2 || a.R + a.rot > a.LW || a.R % 2 || a.rot % 2 ||
      a.LW % 2)
    return -1;
  if (f32) lat_prep_t<float>(a, st);
  else lat_prep_t<bf16_t>(a, st);
  return (int)hipGetLastError();
}

__global__ __launch_bounds__(256) void latent_gather_kernel(u32x4* __restrict__ out,
                                                            const u32x4* __restrict__ cache,
                                                            const int64_t* __restrict__ slots,
                                                            int64_t nvec, int vpr) {
  const int64_t v = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (v >= nvec) return;
  const int64_t row = v / vpr;
  const int64_t slot = slots[row];
  u32x4 x = {0u, 0u, 0u, 0u};
  if (slot >= 0) x = cache[slot * vpr + (v - row * vpr)];
  out[v] = x;
}

int launch_latent_gather(void* out, const void* cache, const int64_t* slots, int rows,
                         int row_bytes, hipStream_t st) {
  if (rows == 0) return 0;
  if (row_bytes % 16) return -1;
  const int vpr = row_bytes / 16;
  const int64_t n = (int64_t)rows * vpr;
  latent_gather_kernel<<<dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st>>>(
      (u32x4*)out, (const u32x4*)cache, slots, n, vpr);
  return (int)hipGetLastError();
}

// ------------------------------------------------------------------ attention, any size
template <class T>
__global__ __launch_bounds__(256) void latent_prefill_any_kernel(LatentPrefillArgs a) {
  const int row = blockIdx.x, h = blockIdx.y;
  // portion of this query row (binary search over the cumulative starts)
  int lo = 0, hi = a.nseq;
  while (hi - lo > 1) {
    const int mid = (lo + hi) >> 1;
    if (a.q_cu[mid] <= row) lo = mid; else hi = mid;
  }
  const int k0 = a.k_cu[lo];
  const int last = a.ctx[lo] + row - a.q_cu[lo];
  const int first = a.window > 0 ? max(0, last - a.window + 1) : 0;
  const T* q = (const T*)a.q + (int64_t)row * a.ldq + h * (a.dim + a.rot);
  const T* kv = (const T*)a.kv + (int64_t)k0 * a.ldkv;
  const T* lat = (const T*)a.lat + (int64_t)k0 * a.LW + a.R;
  attend_any<T>(first, last + 1, a.vdim, a.sink != nullptr, a.sink ? a.sink[h] : 0.f,
                head_gate<T>(a.gate, (int64_t)row * a.ldg + h),
                (T*)a.out + (int64_t)row * a.ldo + h * a.vdim,
                [&](int j) {
                  const T* k = kv + (int64_t)j * a.ldkv + h * a.dim;
                  float s = 0.f;
                  for (int i = 0; i < a.dim; ++i) s += to_f32(q[i]) * to_f32(k[i]);
                  const T* r = lat + (int64_t)j * a.LW;
                  for (int i = 0; i < a.rot; ++i) s += to_f32(q[a.dim + i]) * to_f32(r[i]);
                  return s * a.scale;
                },
                [&](int j, int d) {
                  return to_f32(kv[(int64_t)j * a.ldkv + a.voff + h * a.vdim + d]);
                });
}

template <class T>
__global__ __launch_bounds__(256) void latent_decode_any_kernel(LatentDecodeArgs a) {
  const int b = blockIdx.x, h = blockIdx.y;
  const int ctx = a.context_lens[b];
  T* out = (T*)a.out + ((int64_t)b * a.H + h) * a.R;
  if (ctx <= 0) {
    for (int i = threadIdx.x; i < a.R; i += 256) out[i] = from_f32<T>(0.f);
    return;
  }
  const int first = a.window > 0 ? max(0, ctx - a.window) : 0;
  const int* bt = a.block_tables + (int64_t)b * a.bt_stride;
  const T* q = (const T*)a.qa + ((int64_t)b * a.H + h) * a.LW;
  const T* cache = (const T*)a.cache;
  auto row = [&](int j) { return cache + ((int64_t)bt[j / kLB] * kLB + j % kLB) * a.LW; };
  attend_any<T>(first, ctx, a.R, a.sink != nullptr, a.sink ? a.sink[h] : 0.f,
                head_gate<T>(a.gate, (int64_t)b * a.ldg + h), out,
                [&](int j) {
                  const T* k = row(j);
                  float s = 0.f;
                  for (int i = 0; i < a.LW; ++i) s += to_f32(q[i]) * to_f32(k[i]);
                  return s * a.scale;
                },
                [&](int j, int d) { return to_f32(row(j)[d]); });
}

// ------------------------------------------------------------------ prompt portions on MFMA
// Workgroup: NW waves, QF x 16 query rows each, one head.  K tile [64 keys][DKP] (per-head part,
// then the shared rotated part) and V tile [64][DVP] in LDS, NB buffers; the next tile's global
// loads are in flight during this tile's MFMAs.  S^T = K Q^T, so its accumulators are the P^T
// operand of O^T = V^T P^T without lane movement.  QF = 2 halves the LDS reads per MFMA; NB = 1
// then leaves room for a second workgroup per CU, whose MFMAs run under this one's softmax.
constexpr int kLK = 64;

template <int DKP, int DVP, int NB>
struct LatLds {
  static constexpr int KROW = DKP + 8;
  static constexpr int VROW = DVP + 16;
  static constexpr int K_ELEMS = kLK * KROW;
  static constexpr int BUF = K_ELEMS + kLK * VROW;
  static constexpr size_t BYTES = (size_t)NB * BUF * 2;
};

template <int DKP, int DVP, int QF, int NW, int NB>
__global__ __launch_bounds__(64 * NW, NB == 1 ? 2 : 1) void latent_prefill_kernel(
    LatentPrefillArgs a) {
  using L = LatLds<DKP, DVP, NB>;
  constexpr int NTHR = 64 * NW;
  constexpr int KS = DKP / 32, NT = DVP / 16;
  constexpr int NK = kLK * (DKP / 8) / NTHR, NV = kLK * (DVP / 8) / NTHR;
  constexpr int QT = 16 * NW * QF;
  static_assert(NK * NTHR == kLK * (DKP / 8) && NV * NTHR == kLK * (DVP / 8), "staging split");
  extern __shared__ __attribute__((aligned(16))) bf16_t lat_lds[];

  const int seq = a.tile_seq[blockIdx.x], q0 = a.tile_q0[blockIdx.x], h = blockIdx.y;
  const int qb = a.q_cu[seq], n = a.q_cu[seq + 1] - qb;
  const int kb0 = a.k_cu[seq], nk = a.k_cu[seq + 1] - kb0;
  const int ctx = a.ctx[seq];
  const int w = wave_id_uniform(), lane = threadIdx.x & 63;
  const int col = lane & 15, g = lane >> 4;
  const int dq = a.dim + a.rot;
  const bf16_t* kvp = (const bf16_t*)a.kv + (int64_t)kb0 * a.ldkv;
  const bf16_t* latp = (const bf16_t*)a.lat + (int64_t)kb0 * a.LW + a.R;
  const int win = a.window > 0 ? a.window : 0x3fffffff;
  const int k_lo = max(0, ctx + q0 - win + 1);
  const int k_hi = min(nk, ctx + min(n, q0 + QT));
  const int t_lo = k_lo / kLK, t_hi = (k_hi + kLK - 1) / kLK;

  bf16x8 kr[NK], vr[NV];
  auto issue = [&](int k0) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int v = threadIdx.x + i * NTHR;
      const int key = v / (DKP / 8), c = (v % (DKP / 8)) * 8;
      bf16x8 x = zero8();
      if (k0 + key < k_hi) {
        if (c < a.dim) x = load_bf16x8(kvp + (int64_t)(k0 + key) * a.ldkv + h * a.dim + c);
        else if (c < dq) x = load_bf16x8(latp + (int64_t)(k0 + key) * a.LW + (c - a.dim));
      }
      kr[i] = x;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = threadIdx.x + i * NTHR;
      const int key = v / (DVP / 8), c = (v % (DVP / 8)) * 8;
      bf16x8 x = zero8();
      if (k0 + key < k_hi && c < a.vdim)
        x = load_bf16x8(kvp + (int64_t)(k0 + key) * a.ldkv + a.voff + h * a.vdim + c);
      vr[i] = x;
    }
  };
  auto commit = [&](bf16_t* kb) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int v = threadIdx.x + i * NTHR;
      store_bf16x8(kb + (v / (DKP / 8)) * L::KROW + (v % (DKP / 8)) * 8, kr[i]);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = threadIdx.x + i * NTHR;
      store_bf16x8(kb + L::K_ELEMS + (v / (DVP / 8)) * L::VROW + (v % (DVP / 8)) * 8, vr[i]);
    }
  };

  if (t_lo < t_hi) issue(t_lo * kLK);
  const int qw = q0 + 16 * QF * w;  // this wave's first query row
  bf16x8 qf[QF][KS];
#pragma unroll
  for (int f = 0; f < QF; ++f) {
    const int qr = qw + 16 * f + col;
    const bf16_t* qp = (const bf16_t*)a.q + (int64_t)(qb + qr) * a.ldq + h * dq;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int c = 32 * s + 8 * g;
      qf[f][s] = qr < n && c < dq ? load_bf16x8(qp + c) : zero8();
    }
  }
  f32x4 o[QF][NT];
  float m[QF], lsum[QF];  // m: running maximum of the unscaled scores
#pragma unroll
  for (int f = 0; f < QF; ++f) {
    m[f] = kNegBig;
    lsum[f] = 0.f;
#pragma unroll
    for (int i = 0; i < NT; ++i) o[f][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }
  const float sl2 = a.scale * kLog2e;
  const int tr_off = ((col >> 2) + 4 * g) * L::VROW + 4 * (col & 3);

  int buf = 0;
  for (int kt = t_lo; kt < t_hi; ++kt) {
    bf16_t* kb = lat_lds + buf * L::BUF;
    const bf16_t* vb = kb + L::K_ELEMS;
    if constexpr (NB == 1) __syncthreads();
    else buf ^= 1;
    commit(kb);
    __syncthreads();
    if (kt + 1 < t_hi) issue((kt + 1) * kLK);
    const int k0 = kt * kLK;
    // nothing of this tile for this wave's queries (causal / window): skip its products
    const int q_first = ctx + qw, q_last = ctx + qw + 16 * QF - 1;
    if (k0 > q_last || k0 + kLK - 1 <= q_first - win) continue;
    const bool whole = k0 + kLK - 1 <= q_first && k0 > q_last - win;

    f32x4 sc[QF][4];
#pragma unroll
    for (int st = 0; st < 4; ++st) {
#pragma unroll
      for (int f = 0; f < QF; ++f) sc[f][st] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const bf16x8 kf = load_bf16x8(kb + (16 * st + col) * L::KROW + 32 * s + 8 * g);
#pragma unroll
        for (int f = 0; f < QF; ++f) sc[f][st] = mfma16(kf, qf[f][s], sc[f][st]);
      }
    }
    if (!whole) {
#pragma unroll
      for (int f = 0; f < QF; ++f) {
        const int qpos = ctx + qw + 16 * f + col;
#pragma unroll
        for (int st = 0; st < 4; ++st)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int key = k0 + 16 * st + 4 * g + r;
            if (key > qpos || key <= qpos - win) sc[f][st][r] = kNegBig;
          }
      }
    }
    bf16x8 pf[QF][2];
    float alpha[QF];
    bool moved = false;
#pragma unroll
    for (int f = 0; f < QF; ++f) {
      float bmax = kNegBig;
#pragma unroll
      for (int st = 0; st < 4; ++st)
#pragma unroll
        for (int r = 0; r < 4; ++r) bmax = fmaxf(bmax, sc[f][st][r]);
      bmax = fmaxf(bmax, __shfl_xor(bmax, 16, 64));
      bmax = fmaxf(bmax, __shfl_xor(bmax, 32, 64));
      const float m_new = fmaxf(m[f], bmax);
      alpha[f] = fast_exp2((m[f] - m_new) * sl2);
      moved |= m_new > m[f];
      m[f] = m_new;
      // a row with no key in any tile so far: offset 0, so that its p are 0 (kNegBig minus a
      // rounded product of itself would not be)
      const float off = m_new > 0.5f * kNegBig ? m_new * sl2 : 0.f;
      float psum = 0.f;
#pragma unroll
      for (int ks = 0; ks < 2; ++ks)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float pa = fast_exp2(sc[f][2 * ks][r] * sl2 - off);
          const float pb = fast_exp2(sc[f][2 * ks + 1][r] * sl2 - off);
          psum += pa + pb;
          pf[f][ks][r] = f2bf(pa);
          pf[f][ks][4 + r] = f2bf(pb);
        }
      lsum[f] = lsum[f] * alpha[f] + psum;
    }
    if (__any(moved)) {
#pragma unroll
      for (int f = 0; f < QF; ++f)
#pragma unroll
        for (int i = 0; i < NT; ++i) o[f][i] *= alpha[f];
    }
#pragma unroll
    for (int i = 0; i < NT; ++i) {
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const bf16x4 lo = lat_read_tr16(vb + tr_off + 32 * ks * L::VROW + 16 * i);
        const bf16x4 hi = lat_read_tr16(vb + tr_off + (32 * ks + 16) * L::VROW + 16 * i);
        bf16x8 vf;
#pragma unroll
        for (int j = 0; j < 4; ++j) { vf[j] = lo[j]; vf[4 + j] = hi[j]; }
#pragma unroll
        for (int f = 0; f < QF; ++f) o[f][i] = mfma16(vf, pf[f][ks], o[f][i]);
      }
    }
  }
#pragma unroll
  for (int f = 0; f < QF; ++f) {
    float l = lsum[f];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (a.sink) l += fast_exp2(a.sink[h] * kLog2e - m[f] * sl2);
    const int qr = qw + 16 * f + col;
    if (qr < n) {
      const float inv = head_gate<bf16_t>(a.gate, (int64_t)(qb + qr) * a.ldg + h) / l;
      bf16_t* op = (bf16_t*)a.out + (int64_t)(qb + qr) * a.ldo + h * a.vdim;
#pragma unroll
      for (int i = 0; i < NT; ++i) {
        const int d = 16 * i + 4 * g;
        if (d < a.vdim) {
          bf16x4 v;
#pragma unroll
          for (int r = 0; r < 4; ++r) v[r] = f2bf(o[f][i][r] * inv);
          *reinterpret_cast<bf16x4*>(op + d) = v;
        }
      }
    }
  }
}

template <int DKP, int DVP, int QF, int NW, int NB>
static int lat_prefill_go(const LatentPrefillArgs& a, hipStream_t st) {
  latent_prefill_kernel<DKP, DVP, QF, NW, NB>
      <<<dim3(a.ntiles, a.H), dim3(64 * NW), LatLds<DKP, DVP, NB>::BYTES, st>>>(a);
  return 0;
}
template <int DKP, int DVP>
static int lat_prefill_q(const LatentPrefillArgs& a, hipStream_t st) {
  if constexpr (DKP <= 192 && DVP <= 128) {
    if (a.qtile == 256) return lat_prefill_go<DKP, DVP, 2, 8, 2>(a, st);
    if (a.qtile == 128) return lat_prefill_go<DKP, DVP, 2, 4, 1>(a, st);
  }
  return a.qtile == 64 ? lat_prefill_go<DKP, DVP, 1, 4, 2>(a, st) : -1;
}
template <int DKP>
static int lat_prefill_v(const LatentPrefillArgs& a, hipStream_t st) {
  if (a.vdim <= 64) return lat_prefill_q<DKP, 64>(a, st);
  if (a.vdim <= 128) return lat_prefill_q<DKP, 128>(a, st);
  return lat_prefill_q<DKP, 256>(a, st);
}

int launch_latent_prefill(int f32, const LatentPrefillArgs& a, hipStream_t st) {
  if (a.nseq == 0 || a.nq == 0) return 0;
  const int dq = a.dim + a.rot;
  const bool mfma = !f32 && a.dim % 8 == 0 && a.rot % 8 == 0 && a.vdim % 8 == 0 && dq <= 256 &&
                    a.vdim <= 256 && a.ldq % 8 == 0 && a.ldkv % 8 == 0 && a.voff % 8 == 0 &&
                    a.R % 8 == 0 && a.LW % 8 == 0 && a.ldo % 4 == 0;
  int rc = 0;
  if (mfma) {
    if (dq <= 64) rc = lat_prefill_v<64>(a, st);
    else if (dq <= 128) rc = lat_prefill_v<128>(a, st);
    else if (dq <= 192) rc = lat_prefill_v<192>(a, st);
    else rc = lat_prefill_v<256>(a, st);
  } else {
    if (a.vdim > 1024) return -1;
    if (f32) latent_prefill_any_kernel<float><<<dim3(a.nq, a.H), dim3(256), 0, st>>>(a);
    else latent_prefill_any_kernel<bf16_t><<<dim3(a.nq, a.H), dim3(256), 0, st>>>(a);
  }
  return rc ? rc : (int)hipGetLastError();
}

// ------------------------------------------------------------------ decode on MFMA
// Workgroup: NH head tiles of 16 x ND slices of the output dims, one wave each; grid
// (sequence, group of 16 NH heads, split of the window).  Every wave of a head tile computes
// the tile's scores (they are cheap beside the block's HBM time) and accumulates its slice of
// O^T = C^T P^T.  RT: the latent size in units of 64 (rounded up to 1, 2, 4, 8).  KSX: the
// exact number of 32-column steps of a cache row with R = 64 RT (branch-free products, loads
// batched ahead of them); 0: both at run time.
constexpr int kLatPad = 8;  // row padding: 16 rows of one b128 column start on distinct banks

template <int RT, int NH, int ND, int KSX>
__global__ __launch_bounds__(64 * NH * ND, 2) void latent_decode_kernel(LatentDecodeArgs a) {
  constexpr int NTHR = 64 * NH * ND;
  constexpr int KSM = KSX ? KSX : 2 * RT + 2;  // 32-column steps of a cache row, at most
  constexpr int NTW = 4 * RT / ND;            // output tiles of 16 dims per wave
  constexpr int NVM = (4 * 32 * KSM + NTHR - 1) / NTHR;
  extern __shared__ __attribute__((aligned(16))) bf16_t lat_lds[];
  const int b = blockIdx.x, sp = blockIdx.z;
  const int w = wave_id_uniform(), lane = threadIdx.x & 63;
  const int hw = w / ND, dw = w % ND;
  const int col = lane & 15, g = lane >> 4;
  const int h = (blockIdx.y * NH + hw) * 16 + col;
  const int LW = KSX ? 32 * KSX : a.LW, R = KSX ? 64 * RT : a.R, ks = LW / 32, row_l = LW + kLatPad, tile_l = kLB * row_l;
  const int ctx = a.context_lens[b];
  if (ctx <= 0) {
    if (sp == 0 && h < a.H)
      for (int i = dw * 4 + g; i < R; i += 4 * ND)
        ((bf16_t*)a.out)[((int64_t)b * a.H + h) * R + i] = f2bf(0.f);
    return;
  }
  const int lo = a.window > 0 ? max(0, ctx - a.window) : 0;
  const int t0 = lo / kLB, t1 = (ctx + kLB - 1) / kLB;
  const int nparts = (t1 - t0 + a.tiles_per_split - 1) / a.tiles_per_split;
  const int tb = t0 + sp * a.tiles_per_split, te = min(t1, tb + a.tiles_per_split);
  if (tb >= te) return;
  const int* bt = a.block_tables + (int64_t)b * a.bt_stride;

  // staging: a block is kLB * LW contiguous elements; vector v goes to its padded LDS row
  const int nv = 4 * LW;
  int dst[NVM];
#pragma unroll
  for (int i = 0; i < NVM; ++i) {
    const int v = threadIdx.x + i * NTHR;
    const int r = v * 8 / LW;
    dst[i] = v * 8 + r * (row_l - LW);
  }
  bf16x8 st[NVM];
  auto issue = [&](int t) {
    const bf16_t* p = (const bf16_t*)a.cache + (int64_t)bt[t] * kLB * LW;
#pragma unroll
    for (int i = 0; i < NVM; ++i) {
      const int v = threadIdx.x + i * NTHR;
      if (v < nv) st[i] = load_bf16x8(p + v * 8);
    }
  };
  auto commit = [&](bf16_t* d) {
#pragma unroll
    for (int i = 0; i < NVM; ++i) {
      const int v = threadIdx.x + i * NTHR;
      if (v < nv) store_bf16x8(d + dst[i], st[i]);
    }
  };
  issue(tb);
  bf16x8 qf[KSM];
  const bf16_t* qp = (const bf16_t*)a.qa + ((int64_t)b * a.H + min(h, a.H - 1)) * LW;
#pragma unroll
  for (int s = 0; s < KSM; ++s)
    qf[s] = h < a.H && s < ks ? load_bf16x8(qp + 32 * s + 8 * g) : zero8();
  f32x4 o[NTW];
#pragma unroll
  for (int i = 0; i < NTW; ++i) o[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  float m = kNegBig, lsum = 0.f;
  const float sl2 = a.scale * kLog2e;
  const int tr_off = ((col >> 2) + 4 * g) * row_l + 4 * (col & 3) + 16 * NTW * dw;

  int buf = 0;
  for (int t = tb; t < te; ++t) {
    bf16_t* kb = lat_lds + buf * tile_l;
    buf ^= 1;
    commit(kb);
    __syncthreads();
    if (t + 1 < te) issue(t + 1);
    // four chains (token half x step parity) hide the MFMA latency
    f32x4 part[2][2];
#pragma unroll
    for (int i = 0; i < 4; ++i) part[i >> 1][i & 1] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < KSM; ++s)
      if (KSX || s < ks) {
#pragma unroll
        for (int h2 = 0; h2 < 2; ++h2)
          part[h2][s & 1] = mfma16(load_bf16x8(kb + (16 * h2 + col) * row_l + 32 * s + 8 * g),
                                   qf[s], part[h2][s & 1]);
      }
    f32x4 sc[2];
#pragma unroll
    for (int h2 = 0; h2 < 2; ++h2) sc[h2] = part[h2][0] + part[h2][1];
    float bmax = kNegBig;
#pragma unroll
    for (int h2 = 0; h2 < 2; ++h2)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int pos = t * kLB + 16 * h2 + 4 * g + r;
        sc[h2][r] = pos >= lo && pos < ctx ? sc[h2][r] * sl2 : kNegBig;
        bmax = fmaxf(bmax, sc[h2][r]);
      }
    bmax = fmaxf(bmax, __shfl_xor(bmax, 16, 64));
    bmax = fmaxf(bmax, __shfl_xor(bmax, 32, 64));
    const float m_new = fmaxf(m, bmax);  // every tile of a split holds a visible token
    const float alpha = fast_exp2(m - m_new);
    const bool moved = __any(m_new > m);
    m = m_new;
    bf16x8 pf;
    float psum = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float pa = fast_exp2(sc[0][r] - m_new), pb = fast_exp2(sc[1][r] - m_new);
      psum += pa + pb;
      pf[r] = f2bf(pa);
      pf[4 + r] = f2bf(pb);
    }
    lsum = lsum * alpha + psum;
    if (moved) {
#pragma unroll
      for (int i = 0; i < NTW; ++i) o[i] *= alpha;
    }
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      if (KSX || 16 * (NTW * dw + i) < R) {
        const bf16x4 x = lat_read_tr16(kb + tr_off + 16 * i);
        const bf16x4 y = lat_read_tr16(kb + tr_off + 16 * row_l + 16 * i);
        bf16x8 vf;
#pragma unroll
        for (int j = 0; j < 4; ++j) { vf[j] = x[j]; vf[4 + j] = y[j]; }
        o[i] = mfma16(vf, pf, o[i]);
      }
    }
  }
  lsum += __shfl_xor(lsum, 16, 64);
  lsum += __shfl_xor(lsum, 32, 64);
  if (h >= a.H) return;
  if (nparts == 1) {
    if (a.sink) lsum += fast_exp2(a.sink[h] * kLog2e - m);
    const float inv = head_gate<bf16_t>(a.gate, (int64_t)b * a.ldg + h) / lsum;
    bf16_t* op = (bf16_t*)a.out + ((int64_t)b * a.H + h) * R;
#pragma unroll
    for (int i = 0; i < NTW; ++i) {
      const int d = 16 * (NTW * dw + i) + 4 * g;
      if (d < R) {
        bf16x4 v;
#pragma unroll
        for (int r = 0; r < 4; ++r) v[r] = f2bf(o[i][r] * inv);
        *reinterpret_cast<bf16x4*>(op + d) = v;
      }
    }
    return;
  }
  const int64_t pi = ((int64_t)b * a.H + h) * a.nsplits + sp;
#pragma unroll
  for (int i = 0; i < NTW; ++i) {
    const int d = 16 * (NTW * dw + i) + 4 * g;
    if (d < R) *reinterpret_cast<f32x4*>(a.part_o + pi * R + d) = o[i];
  }
  if (dw == 0 && g == 0) {
    a.part_ml[2 * pi] = m;
    a.part_ml[2 * pi + 1] = lsum;
  }
}

// Merge of the window splits (and the sink): one workgroup per (sequence, head).
__global__ __launch_bounds__(128) void latent_merge_kernel(LatentDecodeArgs a) {
  const int b = blockIdx.x, h = blockIdx.y;
  const int ctx = a.context_lens[b];
  if (ctx <= 0) return;
  const int lo = a.window > 0 ? max(0, ctx - a.window) : 0;
  const int nt = (ctx + kLB - 1) / kLB - lo / kLB;
  const int nparts = (nt + a.tiles_per_split - 1) / a.tiles_per_split;
  if (nparts == 1) return;
  const int64_t pi = ((int64_t)b * a.H + h) * a.nsplits;
  float m = kNegBig;
  for (int p = 0; p < nparts; ++p) m = fmaxf(m, a.part_ml[2 * (pi + p)]);
  float l = a.sink ? fast_exp2(a.sink[h] * kLog2e - m) : 0.f;
  for (int p = 0; p < nparts; ++p)
    l += a.part_ml[2 * (pi + p) + 1] * fast_exp2(a.part_ml[2 * (pi + p)] - m);
  const float inv = head_gate<bf16_t>(a.gate, (int64_t)b * a.ldg + h) / l;
  for (int d = threadIdx.x * 4; d < a.R; d += 512) {
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
    for (int p = 0; p < nparts; ++p)
      s += *reinterpret_cast<const f32x4*>(a.part_o + (pi + p) * a.R + d) *
           fast_exp2(a.part_ml[2 * (pi + p)] - m);
    bf16x4 v;
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = f2bf(s[r] * inv);
    *reinterpret_cast<bf16x4*>((bf16_t*)a.out + ((int64_t)b * a.H + h) * a.R + d) = v;
  }
}

template <int RT, int NH, int ND>
static void lat_decode_go(const LatentDecodeArgs& a, hipStream_t st) {
  const size_t lds = (size_t)2 * kLB * (a.LW + kLatPad) * 2;
  const dim3 grid(a.B, (a.H + 16 * NH - 1) / (16 * NH), a.nsplits), block(64 * NH * ND);
  if constexpr (RT >= 4) {
    if (a.R == 64 * RT && a.LW == 32 * (2 * RT + 2)) {
      latent_decode_kernel<RT, NH, ND, 2 * RT + 2><<<grid, block, lds, st>>>(a);
      return;
    }
    if (a.R == 64 * RT && a.LW == 32 * (2 * RT + 1)) {
      latent_decode_kernel<RT, NH, ND, 2 * RT + 1><<<grid, block, lds, st>>>(a);
      return;
    }
  }
  latent_decode_kernel<RT, NH, ND, 0><<<grid, block, lds, st>>>(a);
}
template <int RT>
static void lat_decode_h(const LatentDecodeArgs& a, hipStream_t st) {
  if (a.H <= 16) lat_decode_go<RT, 1, 4>(a, st);
  else if (a.H <= 32) lat_decode_go<RT, 2, 2>(a, st);
  else lat_decode_go<RT, 4, 2>(a, st);
}

int launch_latent_decode(int f32, const LatentDecodeArgs& a, hipStream_t st) {
  if (a.B == 0) return 0;
  const int ks = a.LW / 32;
  const int need = std::max((a.R + 63) / 64, (ks - 1) / 2);
  if (!f32 && a.R % 8 == 0 && a.LW % 32 == 0 && need <= 8 && a.R <= 512) {
    if (need <= 1) lat_decode_h<1>(a, st);
    else if (need <= 2) lat_decode_h<2>(a, st);
    else if (need <= 4) lat_decode_h<4>(a, st);
    else lat_decode_h<8>(a, st);
    if (a.nsplits > 1) latent_merge_kernel<<<dim3(a.B, a.H), dim3(128), 0, st>>>(a);
  } else {
    if (a.R > 1024) return -1;
    if (f32) latent_decode_any_kernel<float><<<dim3(a.B, a.H), dim3(256), 0, st>>>(a);
    else latent_decode_any_kernel<bf16_t><<<dim3(a.B, a.H), dim3(256), 0, st>>>(a);
  }
  return (int)hipGetLastError();
}

// ------------------------------------------------------------------ per-head projections
// y[b, h, :] = W[h] x[b, h, :], W [H, N, K].  MFMA: 16 output dims per wave, 64 batch rows per
// workgroup sharing each weight fragment; operands straight from global memory (the weights
// are read once per 64 rows and stay in L2).
// WHOLE: K % 128 == 0 - four steps' loads ahead of their products.
template <int NBT, bool WHOLE>
__global__ __launch_bounds__(256) void head_gemm_kernel(
    bf16_t* __restrict__ y, const bf16_t* __restrict__ x, const bf16_t* __restrict__ w, int B,
    int N, int K, int64_t yb, int64_t yh, int64_t xb, int64_t xh) {
  const int h = blockIdx.z, b0 = blockIdx.y * 16 * NBT;
  const int wv = wave_id_uniform(), lane = threadIdx.x & 63;
  const int col = lane & 15, g = lane >> 4;
  const int n0 = (blockIdx.x * 4 + wv) * 16;
  if (n0 >= N) return;
  const bf16_t* wr = w + ((int64_t)h * N + min(n0 + col, N - 1)) * K;
  const bf16_t* xr[NBT];
#pragma unroll
  for (int i = 0; i < NBT; ++i) xr[i] = x + (int64_t)min(b0 + 16 * i + col, B - 1) * xb + h * xh;
  f32x4 acc[NBT];
#pragma unroll
  for (int i = 0; i < NBT; ++i) acc[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  if constexpr (WHOLE) {
    for (int k = 0; k < K; k += 128) {
      bf16x8 wf[4], xf[4][NBT];
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        wf[s] = load_bf16x8(wr + k + 32 * s + 8 * g);
#pragma unroll
        for (int i = 0; i < NBT; ++i) xf[s][i] = load_bf16x8(xr[i] + k + 32 * s + 8 * g);
      }
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int i = 0; i < NBT; ++i) acc[i] = mfma16(wf[s], xf[s][i], acc[i]);
    }
  } else {
    for (int k = 0; k < K; k += 32) {
      const int c = k + 8 * g;
      const bool in = c < K;
      const bf16x8 wf = in ? load_bf16x8(wr + c) : zero8();
#pragma unroll
      for (int i = 0; i < NBT; ++i)
        acc[i] = mfma16(wf, in ? load_bf16x8(xr[i] + c) : zero8(), acc[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < NBT; ++i) {
    const int b = b0 + 16 * i + col, n = n0 + 4 * g;
    if (b < B && n < N) {
      bf16x4 v;
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = f2bf(acc[i][r]);
      *reinterpret_cast<bf16x4*>(y + b * yb + h * yh + n) = v;
    }
  }
}

template <int NBT>
static void head_gemm_go(bf16_t* y, const bf16_t* x, const bf16_t* w, int B, int H, int N, int K,
                         int64_t yb, int64_t yh, int64_t xb, int64_t xh, hipStream_t st) {
  const dim3 grid((N + 63) / 64, (B + 16 * NBT - 1) / (16 * NBT), H);
  if (K % 128 == 0)
    head_gemm_kernel<NBT, true><<<grid, dim3(256), 0, st>>>(y, x, w, B, N, K, yb, yh, xb, xh);
  else
    head_gemm_kernel<NBT, false><<<grid, dim3(256), 0, st>>>(y, x, w, B, N, K, yb, yh, xb, xh);
}

template <class T>
__global__ __launch_bounds__(256) void head_gemm_any_kernel(
    T* __restrict__ y, const T* __restrict__ x, const T* __restrict__ w, int N, int K, int64_t yb,
    int64_t yh, int64_t xb, int64_t xh) {
  const int b = blockIdx.x, h = blockIdx.y, n = blockIdx.z * 256 + threadIdx.x;
  if (n >= N) return;
  const T* xr = x + b * xb + h * xh;
  const T* wr = w + ((int64_t)h * N + n) * K;
  float s = 0.f;
  for (int k = 0; k < K; ++k) s += to_f32(xr[k]) * to_f32(wr[k]);
  y[b * yb + h * yh + n] = from_f32<T>(s);
}

int launch_head_gemm(int f32, void* y, const void* x, const void* w, int B, int H, int N, int K,
                     int64_t yb, int64_t yh, int64_t xb, int64_t xh, hipStream_t st) {
  if (B == 0) return 0;
  if (!f32 && K % 8 == 0 && N % 4 == 0 && yb % 4 == 0 && yh % 4 == 0 && xb % 8 == 0 &&
      xh % 8 == 0) {
    const bf16_t *xx = (const bf16_t*)x, *ww = (const bf16_t*)w;
    if (B <= 16) head_gemm_go<1>((bf16_t*)y, xx, ww, B, H, N, K, yb, yh, xb, xh, st);
    else if (B <= 32) head_gemm_go<2>((bf16_t*)y, xx, ww, B, H, N, K, yb, yh, xb, xh, st);
    else head_gemm_go<4>((bf16_t*)y, xx, ww, B, H, N, K, yb, yh, xb, xh, st);
  } else {
    const dim3 grid(B, H, (N + 255) / 256);
    if (f32)
      head_gemm_any_kernel<float><<<grid, dim3(256), 0, st>>>(
          (float*)y, (const float*)x, (const float*)w, N, K, yb, yh, xb, xh);
    else
      head_gemm_any_kernel<bf16_t><<<grid, dim3(256), 0, st>>>(
          (bf16_t*)y, (const bf16_t*)x, (const bf16_t*)w, N, K, yb, yh, xb, xh);
  }
  return (int)hipGetLastError();
}

// dynamic LDS above 64 KB
template <int DKP, int DVP, int QF, int NW, int NB>
static int lat_prefill_attr() {
  return (int)hipFuncSetAttribute((const void*)latent_prefill_kernel<DKP, DVP, QF, NW, NB>,
                                  hipFuncAttributeMaxDynamicSharedMemorySize,
                                  (int)LatLds<DKP, DVP, NB>::BYTES);
}
template <int DKP, int DVP>
static int lat_prefill_lds() {
  int e = lat_prefill_attr<DKP, DVP, 1, 4, 2>();
  if constexpr (DKP <= 192 && DVP <= 128) {
    if (!e) e = lat_prefill_attr<DKP, DVP, 2, 8, 2>();
    if (!e) e = lat_prefill_attr<DKP, DVP, 2, 4, 1>();
  }
  return e;
}
template <int DKP>
static int lat_prefill_lds_v() {
  int e = lat_prefill_lds<DKP, 64>();
  if (!e) e = lat_prefill_lds<DKP, 128>();
  if (!e) e = lat_prefill_lds<DKP, 256>();
  return e;
}
template <int NH, int ND, int KSX>
static int lat_decode_attr() {
  return (int)hipFuncSetAttribute((const void*)latent_decode_kernel<8, NH, ND, KSX>,
                                  hipFuncAttributeMaxDynamicSharedMemorySize,
                                  2 * kLB * (18 * 32 + kLatPad) * 2);
}
template <int NH, int ND>
static int lat_decode_lds() {
  int e = lat_decode_attr<NH, ND, 0>();
  if (!e) e = lat_decode_attr<NH, ND, 17>();
  if (!e) e = lat_decode_attr<NH, ND, 18>();
  return e;
}
int configure_latent() {
  int e = lat_prefill_lds_v<64>();
  if (!e) e = lat_prefill_lds_v<128>();
  if (!e) e = lat_prefill_lds_v<192>();
  if (!e) e = lat_prefill_lds_v<256>();
  if (!e) e = lat_decode_lds<1, 4>();
  if (!e) e = lat_decode_lds<2, 2>();
  if (!e) e = lat_decode_lds<4, 2>();
  return e;
}

}  // namespace drtc
