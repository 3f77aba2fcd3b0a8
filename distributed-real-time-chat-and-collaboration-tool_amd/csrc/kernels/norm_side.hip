// The 32-bit residual stream of joint layers (gfx950).
//
//   side_norm   h += y / sqrt(mean(y^2) + eps) * yw   (a token's input to the layer before; optional)
//               h  = embed_scale * embed[ids]         (instead, at the first layer)
//               out = (h - mean(h)) / sqrt(var(h) + eps) * w
//   stream_add  h += y; the stream in the activation type
//   side_gate   out = gelu_tanh(z) * embed[ids, part of a layer]; and, for decode-sized batches, the
//               same with z = x . w^T formed in the kernel
//
// side_norm: one workgroup per row, 8 elements to a lane and step, held in registers from the add
// to the scaling, so that the variance is the mean of squared deviations.
#include "hybrid_launchers.h"
#include "typed.h"

namespace drtc {

// Sum over the workgroup with one barrier; `red` holds 16 floats, not written again before another
// barrier.
DRTC_DEVICE float sum_once(float v, float* red) {
  const int nw = blockDim.x >> 6;
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
  for (int i = 0; i < nw; ++i) s += red[i];
  return s;
}

template <class T, int NV>
__global__ __launch_bounds__(256) void side_norm_kernel(SideNormArgs a) {
  __shared__ float red[3][16];
  const int row = blockIdx.x, tid = threadIdx.x, nt = blockDim.x, nvec = a.W / 8;
  float* h = a.h + (int64_t)row * a.W;
  float x[NV][8];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int v = tid + i * nt;
#pragma unroll
    for (int j = 0; j < 8; ++j) x[i][j] = 0.f;
    if (v >= nvec) continue;
    if (a.ids) {
      load8(x[i], (const T*)a.embed + (int64_t)a.ids[row] * a.W + v * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] *= a.embed_scale;
      store8(h + v * 8, x[i]);
    } else {
      load8(x[i], h + v * 8);
    }
  }
  if (a.y) {
    float y[NV][8], ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = tid + i * nt;
#pragma unroll
      for (int j = 0; j < 8; ++j) y[i][j] = 0.f;
      if (v < nvec) load8(y[i], (const T*)a.y + (int64_t)row * a.ldy + v * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += y[i][j] * y[i][j];
    }
    const float r = 1.f / sqrtf(sum_once(ss, red[0]) / (float)a.W + a.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int v = tid + i * nt;
      if (v >= nvec) continue;
      float w[8];
      load8(w, a.yw + v * 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] += y[i][j] * r * w[j];
      store8(h + v * 8, x[i]);
    }
  }
  float s = 0.f, sd = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j) s += x[i][j];
  const float mean = sum_once(s, red[1]) / (float)a.W;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    if (tid + i * nt >= nvec) continue;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      x[i][j] -= mean;
      sd += x[i][j] * x[i][j];
    }
  }
  const float r = 1.f / sqrtf(sum_once(sd, red[2]) / (float)a.W + a.eps);
  T* out = (T*)a.out + (int64_t)row * a.ldo;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int v = tid + i * nt;
    if (v >= nvec) continue;
    float w[8];
    load8(w, a.w + v * 8);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[i][j] *= r * w[j];
    store8(out + v * 8, x[i]);
  }
  for (int c = a.W + tid; c < a.ldo; c += nt) out[c] = from_f32<T>(0.f);
}

// Any width: the row in LDS.
template <class T>
__global__ __launch_bounds__(256) void side_norm_any_kernel(SideNormArgs a) {
  extern __shared__ float sn_row[];
  __shared__ float red[3][16];
  const int row = blockIdx.x, tid = threadIdx.x;
  float* h = a.h + (int64_t)row * a.W;
  const T* y = (const T*)a.y + (int64_t)row * a.ldy;
  float r = 0.f;
  if (a.y) {
    float ss = 0.f;
    for (int c = tid; c < a.W; c += 256) ss += to_f32(y[c]) * to_f32(y[c]);
    r = 1.f / sqrtf(sum_once(ss, red[0]) / (float)a.W + a.eps);
  }
  float s = 0.f, sd = 0.f;
  for (int c = tid; c < a.W; c += 256) {
    float x = a.ids ? to_f32(((const T*)a.embed)[(int64_t)a.ids[row] * a.W + c]) * a.embed_scale : h[c];
    if (a.y) x += to_f32(y[c]) * r * a.yw[c];
    if (a.ids || a.y) h[c] = x;
    sn_row[c] = x;  // read back by this thread only
    s += x;
  }
  const float mean = sum_once(s, red[1]) / (float)a.W;
  for (int c = tid; c < a.W; c += 256) sd += (sn_row[c] - mean) * (sn_row[c] - mean);
  r = 1.f / sqrtf(sum_once(sd, red[2]) / (float)a.W + a.eps);
  T* out = (T*)a.out + (int64_t)row * a.ldo;
  for (int c = tid; c < a.ldo; c += 256)
    out[c] = from_f32<T>(c < a.W ? (sn_row[c] - mean) * r * a.w[c] : 0.f);
}

template <class T>
static int side_norm_t(const SideNormArgs& a, hipStream_t st) {
  const int nvec = a.W / 8, nt = nvec >= 256 ? 256 : (nvec + 63) / 64 * 64;
  const int nv = (nvec + nt - 1) / (nt ? nt : 1);
  const dim3 grid(a.rows), blk(nt);
  if (a.W % 8 || a.ldo % 8 || a.ldy % 8)
    side_norm_any_kernel<T><<<grid, dim3(256), 4 * a.W, st>>>(a);
  else if (nv == 1) side_norm_kernel<T, 1><<<grid, blk, 0, st>>>(a);
  else if (nv == 2) side_norm_kernel<T, 2><<<grid, blk, 0, st>>>(a);
  else if (nv <= 4) side_norm_kernel<T, 4><<<grid, blk, 0, st>>>(a);
  else side_norm_kernel<T, 8><<<grid, blk, 0, st>>>(a);
  return (int)hipGetLastError();
}

int launch_side_norm(int f32, const SideNormArgs& a, hipStream_t st) {
  if (a.rows == 0) return 0;
  if (a.W < 1 || a.W > 16384 || a.ldo < a.W) return -1;
  return f32 ? side_norm_t<float>(a, st) : side_norm_t<bf16_t>(a, st);
}

// ------------------------------------------------------------------ elementwise
template <class T>
__global__ __launch_bounds__(256) void stream_add_kernel(T* __restrict__ out, float* __restrict__ h,
                                                         const T* __restrict__ y, int64_t ldy,
                                                         int64_t n, int W, bool vec) {
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * (vec ? 8 : 1);
  if (i >= n) return;
  const int64_t row = i / W, c = i - row * W;
  if (vec) {
    float x[8], d[8];
    load8(x, h + i);
    load8(d, y + row * ldy + c);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] += d[j];
    store8(h + i, x);
    if constexpr (sizeof(T) == 2) store8(out + i, x);
  } else {
    const float x = h[i] + to_f32(y[row * ldy + c]);
    h[i] = x;
    if constexpr (sizeof(T) == 2) out[i] = from_f32<T>(x);
  }
}

// fp32: the stream itself is the second output
int launch_stream_add(int f32, void* out, float* h, const void* y, int64_t ldy, int rows, int W,
                      hipStream_t st) {
  const int64_t n = (int64_t)rows * W;
  if (n == 0) return 0;
  const bool vec = W % 8 == 0 && ldy % 8 == 0 && (uintptr_t)y % 16 == 0;
  const int64_t per = 256 * (vec ? 8 : 1);
  const dim3 grid((unsigned)((n + per - 1) / per));
  if (f32) stream_add_kernel<float><<<grid, dim3(256), 0, st>>>((float*)out, h, (const float*)y, ldy, n, W, vec);
  else stream_add_kernel<bf16_t><<<grid, dim3(256), 0, st>>>((bf16_t*)out, h, (const bf16_t*)y, ldy, n, W, vec);
  return (int)hipGetLastError();
}

template <class T>
DRTC_DEVICE float side_gelu(float z) {
  if constexpr (sizeof(T) == 2) return act_value<1>(z);
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

template <class T, int V>
__global__ __launch_bounds__(256) void side_gate_kernel(T* __restrict__ out, const T* __restrict__ z,
                                                        const T* __restrict__ embed, int64_t lde,
                                                        int off, const int* __restrict__ ids,
                                                        int64_t n, int dim) {
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= n) return;
  const int64_t row = i / dim;
  const int c = (int)(i - row * dim);
  const T* e = embed + (int64_t)ids[row] * lde + off + c;
  if constexpr (V == 8) {
    float x[8], y[8];
    load8(x, z + i);
    load8(y, e);
#pragma unroll
    for (int j = 0; j < 8; ++j) x[j] = side_gelu<T>(x[j]) * y[j];
    store8(out + i, x);
  } else {
    out[i] = from_f32<T>(side_gelu<T>(to_f32(z[i])) * to_f32(*e));
  }
}

template <class T>
static void side_gate_t(void* out, const void* z, const void* embed, int64_t lde, int off,
                        const int* ids, int64_t n, int dim, hipStream_t st) {
  if (dim % 8 == 0 && lde % 8 == 0 && off % 8 == 0)
    side_gate_kernel<T, 8><<<dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0, st>>>(
        (T*)out, (const T*)z, (const T*)embed, lde, off, ids, n, dim);
  else
    side_gate_kernel<T, 1><<<dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st>>>(
        (T*)out, (const T*)z, (const T*)embed, lde, off, ids, n, dim);
}

int launch_side_gate(int f32, void* out, const void* z, const void* embed, int64_t lde, int off,
                     const int* ids, int rows, int dim, hipStream_t st) {
  const int64_t n = (int64_t)rows * dim;
  if (n == 0) return 0;
  if (off < 0 || off + dim > lde) return -1;
  if (f32) side_gate_t<float>(out, z, embed, lde, off, ids, n, dim, st);
  else side_gate_t<bf16_t>(out, z, embed, lde, off, ids, n, dim, st);
  return (int)hipGetLastError();
}

// z = x . w^T, gated: 16 tokens x 16 CT columns to a workgroup, whose 8 waves take every eighth
// 32-column step of the reduction; operands straight from global memory.
constexpr int kSideWaves = 8;
template <int CT>
__global__ __launch_bounds__(64 * kSideWaves) void side_gate_gemm_kernel(
    bf16_t* __restrict__ out, const bf16_t* __restrict__ x, const bf16_t* __restrict__ w,
    const bf16_t* __restrict__ embed, int64_t lde, int off, const int* __restrict__ ids, int T, int N,
    int K) {
  __shared__ float part[kSideWaves][16][16 * CT + 1];
  const int t0 = blockIdx.x * 16, n0 = blockIdx.y * 16 * CT, lane = threadIdx.x & 63;
  const int wv = wave_id_uniform(), col = lane & 15, g = lane >> 4;
  const bf16_t* xr = x + (int64_t)min(t0 + col, T - 1) * K;
  f32x4 acc[CT];
#pragma unroll
  for (int i = 0; i < CT; ++i) acc[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  bf16x8 zero;
#pragma unroll
  for (int j = 0; j < 8; ++j) zero[j] = f2bf(0.f);
  // this thread's output and its token's input, on the way during the products
  static_assert(CT <= 2, "an output to a thread");
  const int ot = threadIdx.x / (16 * CT), on = threadIdx.x % (16 * CT);
  const bool mine = threadIdx.x < 256 * CT && t0 + ot < T && n0 + on < N;
  const bf16_t e = mine ? embed[(int64_t)ids[t0 + ot] * lde + off + n0 + on] : zero[0];
  // U steps' loads ahead of their products; steps behind the end add zeros
  constexpr int U = 16;
  for (int c0 = 32 * wv; c0 < K; c0 += 32 * kSideWaves * U) {
    bf16x8 b[U], a[U][CT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = min(c0 + 32 * kSideWaves * u + 8 * g, K - 8);
      b[u] = load_bf16x8(xr + c);
#pragma unroll
      for (int i = 0; i < CT; ++i)
        a[u][i] = load_bf16x8(w + (int64_t)min(n0 + 16 * i + col, N - 1) * K + c);
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      b[u] = c0 + 32 * kSideWaves * u + 8 * g < K ? b[u] : zero;
#pragma unroll
      for (int i = 0; i < CT; ++i) acc[i] = mfma16(a[u][i], b[u], acc[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < CT; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) part[wv][col][16 * i + 4 * g + r] = acc[i][r];
  __syncthreads();
  if (!mine) return;
  float z = part[0][ot][on];
#pragma unroll
  for (int o = 1; o < kSideWaves; ++o) z += part[o][ot][on];
  out[(int64_t)(t0 + ot) * N + n0 + on] = f2bf(act_value<1>(z) * bf2f(e));
}

int launch_side_gate_gemm(void* out, const void* x, const void* w, const void* embed, int64_t lde,
                          int off, const int* ids, int T, int N, int K, hipStream_t st) {
  if (T == 0 || N == 0) return 0;
  if (K < 8 || K % 8 || off < 0 || off + N > lde) return -1;
  const bf16_t *xx = (const bf16_t*)x, *ww = (const bf16_t*)w, *ee = (const bf16_t*)embed;
  const dim3 blk(64 * kSideWaves);
  if (T <= 128)
    side_gate_gemm_kernel<1><<<dim3((T + 15) / 16, (N + 15) / 16), blk, 0, st>>>(
        (bf16_t*)out, xx, ww, ee, lde, off, ids, T, N, K);
  else
    side_gate_gemm_kernel<2><<<dim3((T + 15) / 16, (N + 31) / 32), blk, 0, st>>>(
        (bf16_t*)out, xx, ww, ee, lde, off, ids, T, N, K);
  return (int)hipGetLastError();
}

}  // namespace drtc
