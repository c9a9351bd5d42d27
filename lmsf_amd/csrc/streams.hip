// A residual of several streams: n rows of W float32 numbers a token, X [N, n, W]. Around a sublayer f with the numbers
// a, b [n] and M [n, n] of its own:
//     u = sum_s a_s X_s;   y = f(norm(u));   X_t <- sum_s M[s, t] X_s + b_t y      (all t at once from the old X)
// One kernel closes a sublayer and opens the next: it brings the streams up to date with the earlier sublayer's y, M and
// b, sums the new ones with the next a and norms the sum (u / rms(u) * w). Every operand is optional: without y the
// streams stay, without w nothing is normed, with ``rows`` only those tokens are computed and the streams are left as
// they were (the end of a model: a = 1 everywhere, and only the rows whose logits are wanted).
// A workgroup a token. Up to eight streams and rows of a multiple of four entries: a thread takes four neighbours of all
// streams at a time and keeps the sum in registers between the update and the norm; else an entry at a time, the sum in
// LDS. Everything is float32 but y and the norm's result, which are in the run's type.
// The reference's residual is one stream (core/src/model_executor/models/llama/llama.rs:286-340).
#include "common.h"
#include "entry_points.h"

#include <math.h>

#define ST_MAX 32          // streams

template <typename T> struct St4;
template <> struct St4<float> {
  static __device__ __forceinline__ void load(const float* p, float* x) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    x[0] = v.x, x[1] = v.y, x[2] = v.z, x[3] = v.w;
  }
  static __device__ __forceinline__ void store(float* p, const float* x) {
    *reinterpret_cast<float4*>(p) = make_float4(x[0], x[1], x[2], x[3]);
  }
};
template <> struct St4<bf16_t> {
  static __device__ __forceinline__ void load(const bf16_t* p, float* x) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    x[0] = __uint_as_float(v.x << 16), x[1] = __uint_as_float(v.x & 0xffff0000u);
    x[2] = __uint_as_float(v.y << 16), x[3] = __uint_as_float(v.y & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float* x) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack2_bf16(x[0], x[1]), pack2_bf16(x[2], x[3]));
  }
};

// NS: the number of streams (a constant, so that they are registers); E: groups of four entries a thread holds
template <typename T, int NS, int E>
__global__ __launch_bounds__(1024) void mix_streams_kernel(float* __restrict__ X, const T* __restrict__ y, long y_stride,
                                                           const float* __restrict__ M, const float* __restrict__ b,
                                                           const float* __restrict__ a, const float* __restrict__ w,
                                                           float eps, const int* __restrict__ rows, T* __restrict__ out,
                                                           int W) {
  __shared__ float red[16];
  const long n = rows ? rows[blockIdx.x] : blockIdx.x;
  float* Xn = X + n * NS * W;
  float x[E][NS][4], yv[E][4], u[E][4];
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int i = (threadIdx.x + e * blockDim.x) * 4;
    if (i < W) {
#pragma unroll
      for (int s = 0; s < NS; ++s) St4<float>::load(Xn + (long)s * W + i, x[e][s]);
      if (y) St4<T>::load(y + n * y_stride + i, yv[e]);
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int i = (threadIdx.x + e * blockDim.x) * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) u[e][j] = 0.f;
    if (i >= W) continue;
    if (y) {
      float r[NS][4];
#pragma unroll
      for (int t = 0; t < NS; ++t) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          float acc = b[t] * yv[e][j];
#pragma unroll
          for (int s = 0; s < NS; ++s) acc = fmaf(M[s * NS + t], x[e][s][j], acc);
          r[t][j] = acc;
        }
        if (!rows) St4<float>::store(Xn + (long)t * W + i, r[t]);
      }
#pragma unroll
      for (int t = 0; t < NS; ++t)
#pragma unroll
        for (int j = 0; j < 4; ++j) x[e][t][j] = r[t][j];
    }
    if (w) {
#pragma unroll
      for (int s = 0; s < NS; ++s)
#pragma unroll
        for (int j = 0; j < 4; ++j) u[e][j] = fmaf(a ? a[s] : 1.f, x[e][s][j], u[e][j]);
#pragma unroll
      for (int j = 0; j < 4; ++j) ss = fmaf(u[e][j], u[e][j], ss);
    }
  }
  if (!w) return;
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)W + eps);
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int i = (threadIdx.x + e * blockDim.x) * 4;
    if (i < W) {
      float wv[4];
      St4<float>::load(w + i, wv);
#pragma unroll
      for (int j = 0; j < 4; ++j) wv[j] *= u[e][j] * inv;
      St4<T>::store(out + (long)blockIdx.x * W + i, wv);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void mix_streams_general_kernel(float* __restrict__ X, int ns, const T* __restrict__ y,
                                                                  long y_stride, const float* __restrict__ M,
                                                                  const float* __restrict__ b, const float* __restrict__ a,
                                                                  const float* __restrict__ w, float eps,
                                                                  const int* __restrict__ rows, T* __restrict__ out,
                                                                  int W) {
  extern __shared__ float u[];       // [W]
  __shared__ float red[16];
  const long n = rows ? rows[blockIdx.x] : blockIdx.x;
  float* Xn = X + n * ns * W;
  float ss = 0.f;
  for (int i = threadIdx.x; i < W; i += 256) {
    float x[ST_MAX];
#pragma unroll
    for (int s = 0; s < ST_MAX; ++s) x[s] = s < ns ? Xn[(long)s * W + i] : 0.f;
    const float yv = y ? to_f32<T>(y[n * y_stride + i]) : 0.f;
    float sum = 0.f;
    for (int t = 0; t < ns; ++t) {
      float v;
      if (y) {
        v = b[t] * yv;
#pragma unroll
        for (int s = 0; s < ST_MAX; ++s)
          if (s < ns) v = fmaf(M[s * ns + t], x[s], v);
        if (!rows) Xn[(long)t * W + i] = v;
      } else {
        v = Xn[(long)t * W + i];
      }
      sum = fmaf(a ? a[t] : 1.f, v, sum);
    }
    u[i] = sum;
    ss = fmaf(sum, sum, ss);
  }
  if (!w) return;
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += 256)      // (each thread reads back what it wrote itself)
    out[(long)blockIdx.x * W + i] = from_f32<T>(w[i] * (u[i] * inv));
}

template <typename T, int NS>
static void mix_streams_launch(float* X, const void* y, long y_stride, const float* M, const float* b, const float* a,
                               const float* w, float eps, const int* rows, void* out, int n_rows, int W,
                               hipStream_t stream) {
  // many rows: small workgroups with two accesses a thread; few rows: as many threads as a row has groups of four
  const int quads = W / 4, per_thread = n_rows >= 512 ? 2 : 1;
  int threads = 64;
  while (threads < 1024 && threads * per_thread < quads) threads *= 2;
  const int need = (quads + threads - 1) / threads;
#define MS(E)                                                                                                       \
  hipLaunchKernelGGL((mix_streams_kernel<T, NS, E>), dim3(n_rows), dim3(threads), 0, stream, X, (const T*)y,        \
                     y_stride, M, b, a, w, eps, rows, (T*)out, W)
  if (need <= 1) MS(1); else if (need <= 2) MS(2); else MS(4);
#undef MS
}

// X float32 [N, ns, W]; y [N, W] of ``dtype`` (null: the streams stay), M [ns, ns] from row to column, b [ns];
// a [ns] (null: ones) and w [W] (null: no result), out [n_rows, W] of ``dtype``; rows int32 [n_rows] (null: rows
// 0 .. n_rows - 1): the tokens to compute, the streams are not written then.
extern "C" int lmsf_mix_streams(float* X, int ns, const void* y, long y_stride, const float* M, const float* b,
                                const float* a, const float* w, float eps, const int* rows, void* out, int dtype,
                                int n_rows, int W, hipStream_t stream) {
  LMSF_CHECK(X && (!y || (M && b)) && (!w || out) && (y || w), "mix_streams: null pointer");
  LMSF_CHECK(dtype == LMSF_F32 || dtype == LMSF_BF16, "mix_streams: unknown dtype code %d", dtype);
  LMSF_CHECK(ns >= 1 && ns <= ST_MAX, "mix_streams: %d streams (at most %d)", ns, ST_MAX);
  LMSF_CHECK(W > 0 && W <= 16384 && (!y || y_stride >= W), "mix_streams: rows of %d entries (at most 16,384)", W);
  if (n_rows <= 0) return 0;
  const bool vec = W % 4 == 0 && ns <= 8 && (!y || y_stride % 4 == 0) && lmsf_aligned16(X) && lmsf_aligned16(y) &&
                   lmsf_aligned16(w) && lmsf_aligned16(out);
#define MS_GO(T)                                                                                                     \
  do {                                                                                                               \
    if (!vec) {                                                                                                      \
      hipLaunchKernelGGL((mix_streams_general_kernel<T>), dim3(n_rows), dim3(256), (size_t)W * 4, stream, X, ns,     \
                         (const T*)y, y_stride, M, b, a, w, eps, rows, (T*)out, W);                                  \
      break;                                                                                                         \
    }                                                                                                                \
    switch (ns) {                                                                                                    \
      case 1: mix_streams_launch<T, 1>(X, y, y_stride, M, b, a, w, eps, rows, out, n_rows, W, stream); break;        \
      case 2: mix_streams_launch<T, 2>(X, y, y_stride, M, b, a, w, eps, rows, out, n_rows, W, stream); break;        \
      case 3: mix_streams_launch<T, 3>(X, y, y_stride, M, b, a, w, eps, rows, out, n_rows, W, stream); break;        \
      case 4: mix_streams_launch<T, 4>(X, y, y_stride, M, b, a, w, eps, rows, out, n_rows, W, stream); break;        \
      case 5: mix_streams_launch<T, 5>(X, y, y_stride, M, b, a, w, eps, rows, out, n_rows, W, stream); break;        \
      case 6: mix_streams_launch<T, 6>(X, y, y_stride, M, b, a, w, eps, rows, out, n_rows, W, stream); break;        \
      case 7: mix_streams_launch<T, 7>(X, y, y_stride, M, b, a, w, eps, rows, out, n_rows, W, stream); break;        \
      default: mix_streams_launch<T, 8>(X, y, y_stride, M, b, a, w, eps, rows, out, n_rows, W, stream); break;       \
    }                                                                                                                \
  } while (0)
  if (dtype == LMSF_F32) MS_GO(float); else MS_GO(bf16_t);
#undef MS_GO
  LMSF_LAUNCH_CHECK("mix_streams");
  return 0;
}

// X[n, s] = scale * table[ids[n]] for every stream s (an id outside the table: zeros, and the flag is raised)
template <typename T>
__global__ __launch_bounds__(256) void stream_embedding_kernel(const int* __restrict__ ids, const T* __restrict__ table,
                                                               float scale, float* __restrict__ X, int ns, int V, int W,
                                                               int* __restrict__ bad_flag) {
  const long n = blockIdx.x;
  const int id = ids[n];
  const bool ok = id >= 0 && id < V;
  if (!ok && threadIdx.x == 0 && blockIdx.y == 0 && bad_flag) atomicOr(bad_flag, 1);
  if (W % 4 == 0) {             // (X and the table begin at multiples of 16 bytes: every row at one of four entries)
    for (int i = (blockIdx.y * 256 + threadIdx.x) * 4; i < W; i += gridDim.y * 1024) {
      float v[4] = {0.f, 0.f, 0.f, 0.f};
      if (ok) St4<T>::load(table + (long)id * W + i, v);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] *= scale;
      for (int s = 0; s < ns; ++s) St4<float>::store(X + (n * ns + s) * W + i, v);
    }
    return;
  }
  for (int i = blockIdx.y * 256 + threadIdx.x; i < W; i += gridDim.y * 256) {
    const float v = ok ? scale * to_f32<T>(table[(long)id * W + i]) : 0.f;
    for (int s = 0; s < ns; ++s) X[(n * ns + s) * W + i] = v;
  }
}

extern "C" int lmsf_stream_embedding(const int* ids, const void* table, int dtype, float scale, float* X, int n_tokens,
                                     int ns, int V, int W, int* bad_flag, hipStream_t stream) {
  LMSF_CHECK(ids && table && X, "stream_embedding: null pointer");
  LMSF_CHECK(dtype == LMSF_F32 || dtype == LMSF_BF16, "stream_embedding: unknown dtype code %d", dtype);
  LMSF_CHECK(ns > 0 && V > 0 && W > 0, "stream_embedding: bad sizes");
  LMSF_CHECK(lmsf_aligned16(X) && lmsf_aligned16(table), "stream_embedding: operands must be 16-byte aligned");
  if (n_tokens <= 0) return 0;
  const dim3 grid(n_tokens, min((W + 1023) / 1024, 64));
  if (dtype == LMSF_F32)
    hipLaunchKernelGGL((stream_embedding_kernel<float>), grid, dim3(256), 0, stream, ids, (const float*)table, scale, X,
                       ns, V, W, bad_flag);
  else
    hipLaunchKernelGGL((stream_embedding_kernel<bf16_t>), grid, dim3(256), 0, stream, ids, (const bf16_t*)table, scale, X,
                       ns, V, W, bad_flag);
  LMSF_LAUNCH_CHECK("stream_embedding");
  return 0;
}
