// RMS norm in groups around a float32 residual stream, with the additions that surround it.
//
// A row of W numbers is cut into ``groups`` equal consecutive parts; part g is divided by
// sqrt(mean(part^2) + eps) and the whole row is multiplied by a weight:  gn(x; w)_i = x_i / rms_g(i) * w_i.
// groups = 1 is the plain RMS norm.
//
// One kernel serves the arrangements in which a layer uses such norms; every operand is optional:
//
//   v = branch ? gn(branch[row]; wb) : 0                    the norm *after* a sublayer
//   r = residual ? residual[src] + v : v                    src = rows ? rows[row] : row
//   residual[row] = r                                       (branch, residual, no rows)
//   hist[k][row] = r;  x = sum_{j<=k} mix[j] hist[j][row];  residual[row] = x      (hist: a weighted average over
//                                                           the results of all layers so far, r being the k-th)
//   out[row] = wn ? gn(x; wn) : x                           the norm *before* the next sublayer
//
// All arithmetic is float32; branch and out are float32 or bfloat16, the weights float32. One workgroup a row
// (256 to 1,024 threads), the row kept in LDS between the passes; the stream's row and the earlier results are asked
// for before the first pass, so that the passes do not each wait for memory.
#include "common.h"

#include <math.h>

#define GN_MAX_THREADS 1024
#define GN_THREADS ((int)blockDim.x)

template <typename T>
__device__ __forceinline__ float gn_load(const void* p, long i) { return to_f32<T>(((const T*)p)[i]); }

// divides the row in LDS by its groups' root mean squares and multiplies by w; ``red`` is block_sum's scratch
__device__ __forceinline__ void gn_normalize(float* row, const float* __restrict__ w, int W, int groups, float eps,
                                             float* red) {
  const int gw = W / groups;
  for (int g = 0; g < groups; ++g) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < gw; i += GN_THREADS) {
      const float x = row[g * gw + i];
      ss += x * x;
    }
    ss = block_sum(ss, red);
    const float rms = sqrtf(ss / (float)gw + eps);
    for (int i = threadIdx.x; i < gw; i += GN_THREADS) row[g * gw + i] = row[g * gw + i] / rms * w[g * gw + i];
  }
  __syncthreads();
}

template <typename TB, typename TO>
__global__ __launch_bounds__(GN_MAX_THREADS) void group_norm_kernel(
    const TB* __restrict__ branch, long branch_stride, const float* __restrict__ wb, float* __restrict__ residual,
    float* __restrict__ hist, long hist_stride, int hist_index, const float* __restrict__ mix,
    const float* __restrict__ wn, TO* __restrict__ out, long out_stride, const int* __restrict__ rows, int W,
    int groups, float eps_b, float eps_n) {
  extern __shared__ float row[];   // [W] the row; [W] the stream's row; [W] the earlier results' share of the average
  float* res = row + W;
  float* before = row + 2 * W;
  __shared__ float red[16];
  const int n = blockIdx.x;
  const int src = rows ? rows[n] : n;
  // everything that comes from memory is asked for at once: the passes below would otherwise each wait for their own
  if (residual)
    for (int i = threadIdx.x; i < W; i += GN_THREADS) res[i] = residual[(long)src * W + i];
  if (hist)
    for (int i = threadIdx.x; i < W; i += GN_THREADS) {
      float x = 0.f;
#pragma unroll 8
      for (int j = 0; j < hist_index; ++j) x += mix[j] * hist[(long)j * hist_stride + (long)n * W + i];
      before[i] = x;
    }
  if (branch) {
    for (int i = threadIdx.x; i < W; i += GN_THREADS) row[i] = to_f32<TB>(branch[(long)n * branch_stride + i]);
    __syncthreads();
    gn_normalize(row, wb, W, groups, eps_b, red);
  }
  // (each thread reads back the entries of res and before that it wrote itself)
  if (residual) {
    const bool store = branch && !rows && !hist;
    for (int i = threadIdx.x; i < W; i += GN_THREADS) {
      const float r = res[i] + (branch ? row[i] : 0.f);
      row[i] = r;
      if (store) residual[(long)n * W + i] = r;
    }
  }
  if (hist) {
    for (int i = threadIdx.x; i < W; i += GN_THREADS) {
      const float r = row[i];
      hist[(long)hist_index * hist_stride + (long)n * W + i] = r;
      const float x = before[i] + mix[hist_index] * r;
      row[i] = x;
      residual[(long)n * W + i] = x;
    }
  }
  if (out) {
    __syncthreads();
    if (wn) gn_normalize(row, wn, W, groups, eps_n, red);
    for (int i = threadIdx.x; i < W; i += GN_THREADS) out[(long)n * out_stride + i] = from_f32<TO>(row[i]);
  }
}

template <typename TB, typename TO>
static void gn_launch(int n_rows, size_t smem, hipStream_t stream, const void* branch, long branch_stride,
                      const float* wb, float* residual, float* hist, long hist_stride, int hist_index,
                      const float* mix, const float* wn, void* out, long out_stride, const int* rows, int W,
                      int groups, float eps_b, float eps_n) {
  // few rows: a row's passes wait for memory one after the other, so many threads with few elements each; many
  // rows fill the chip with smaller workgroups
  const int threads = n_rows >= 1024 || W <= 256 ? 256 : W <= 1024 ? 512 : 1024;
  hipLaunchKernelGGL((group_norm_kernel<TB, TO>), dim3(n_rows), dim3(threads), smem, stream, (const TB*)branch,
                     branch_stride, wb, residual, hist, hist_stride, hist_index, mix, wn, (TO*)out, out_stride, rows,
                     W, groups, eps_b, eps_n);
}

extern "C" int lmsf_group_norm(const void* branch, int branch_dtype, long branch_stride, const float* wb,
                               float* residual, float* hist, long hist_stride, int hist_index, const float* mix,
                               const float* wn, void* out, int out_dtype, long out_stride, const int* rows,
                               int n_rows, int W, int groups, float eps_b, float eps_n, hipStream_t stream) {
  LMSF_CHECK(branch || residual, "group_norm: neither a branch nor a residual");
  LMSF_CHECK(W > 0 && groups > 0 && W % groups == 0, "group_norm: %d columns do not split into %d groups", W, groups);
  LMSF_CHECK((size_t)W * 12 <= 160 * 1024 - 256, "group_norm: three rows of %d columns do not fit LDS", W);
  LMSF_CHECK(!branch || wb, "group_norm: a branch needs its weight");
  LMSF_CHECK(!branch || branch_stride >= W, "group_norm: branch rows overlap");
  LMSF_CHECK(!out || out_stride >= W, "group_norm: output rows overlap");
  LMSF_CHECK(!hist || (residual && mix && hist_index >= 0 && hist_stride >= (long)n_rows * W && !rows),
             "group_norm: the running average needs a residual, its weights and whole rows");
  LMSF_CHECK(branch_dtype == LMSF_F32 || branch_dtype == LMSF_BF16, "group_norm: unknown dtype code %d", branch_dtype);
  LMSF_CHECK(out_dtype == LMSF_F32 || out_dtype == LMSF_BF16, "group_norm: unknown dtype code %d", out_dtype);
  if (n_rows <= 0) return 0;
  const size_t smem = (size_t)W * 12;
  if (smem > 64 * 1024) {
    // (once per instantiation would do; the call is cheap)
    hipFuncSetAttribute((const void*)group_norm_kernel<float, float>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    hipFuncSetAttribute((const void*)group_norm_kernel<float, bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    hipFuncSetAttribute((const void*)group_norm_kernel<bf16_t, float>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
    hipFuncSetAttribute((const void*)group_norm_kernel<bf16_t, bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  }
#define GN_ARGS n_rows, smem, stream, branch, branch_stride, wb, residual, hist, hist_stride, hist_index, mix, wn, out, \
                out_stride, rows, W, groups, eps_b, eps_n
  if (branch_dtype == LMSF_F32 && out_dtype == LMSF_F32) gn_launch<float, float>(GN_ARGS);
  else if (branch_dtype == LMSF_F32) gn_launch<float, bf16_t>(GN_ARGS);
  else if (out_dtype == LMSF_F32) gn_launch<bf16_t, float>(GN_ARGS);
  else gn_launch<bf16_t, bf16_t>(GN_ARGS);
#undef GN_ARGS
  LMSF_LAUNCH_CHECK("group_norm");
  return 0;
}

// ---------------------------------------------------------------- a sublayer's output, normed, into the stream
//
//   v = b ? scale (a / rms(a) * wa + b / rms(b) * wb) : a;    residual += v / rms(v) * wn;    out = residual in T
//
// (two mixers side by side are joined on the way: nothing of v goes through memory). A workgroup a row, the row in
// registers, four neighbours an access; everything that comes from memory is asked for before the first sum.

template <typename T> struct Na4;
template <> struct Na4<float> {
  static __device__ __forceinline__ void load(const float* p, float* x) {
    const float4 v = *reinterpret_cast<const float4*>(p);
    x[0] = v.x; x[1] = v.y; x[2] = v.z; x[3] = v.w;
  }
  static __device__ __forceinline__ void store(float* p, const float* x) {
    *reinterpret_cast<float4*>(p) = make_float4(x[0], x[1], x[2], x[3]);
  }
};
template <> struct Na4<bf16_t> {
  static __device__ __forceinline__ void load(const bf16_t* p, float* x) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    x[0] = __uint_as_float(v.x << 16); x[1] = __uint_as_float(v.x & 0xffff0000u);
    x[2] = __uint_as_float(v.y << 16); x[3] = __uint_as_float(v.y & 0xffff0000u);
  }
  static __device__ __forceinline__ void store(bf16_t* p, const float* x) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack2_bf16(x[0], x[1]), pack2_bf16(x[2], x[3]));
  }
};

// E: groups of four entries a thread holds
template <typename T, bool PAIR, int E>
__global__ __launch_bounds__(1024) void norm_add_kernel(const T* __restrict__ a, long a_stride, const T* __restrict__ b,
                                                        long b_stride, const float* __restrict__ wa,
                                                        const float* __restrict__ wb, float eps_pair, float scale,
                                                        const float* __restrict__ wn, float eps,
                                                        float* __restrict__ residual, T* __restrict__ out, int W) {
  __shared__ float red[3][16];
  const long n = blockIdx.x;
  const int wave = threadIdx.x / LMSF_WAVE, lane = threadIdx.x % LMSF_WAVE, n_waves = blockDim.x / LMSF_WAVE;
  float va[E][4], vb[E][4], res[E][4], w[E][4];
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int i = (threadIdx.x + e * blockDim.x) * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) va[e][j] = vb[e][j] = 0.f;
    if (i < W) {
      Na4<T>::load(a + n * a_stride + i, va[e]);
      if (PAIR) Na4<T>::load(b + n * b_stride + i, vb[e]);
      Na4<float>::load(residual + n * W + i, res[e]);
      Na4<float>::load(wn + i, w[e]);
    }
  }
  if (PAIR) {
    float sa = 0.f, sb = 0.f;
#pragma unroll
    for (int e = 0; e < E; ++e)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        sa = fmaf(va[e][j], va[e][j], sa);
        sb = fmaf(vb[e][j], vb[e][j], sb);
      }
    sa = wave_sum(sa);
    sb = wave_sum(sb);
    if (lane == 0) {
      red[0][wave] = sa;
      red[1][wave] = sb;
    }
    __syncthreads();
    sa = sb = 0.f;
    for (int k = 0; k < n_waves; ++k) {
      sa += red[0][k];
      sb += red[1][k];
    }
    const float ia = scale / sqrtf(sa / (float)W + eps_pair), ib = scale / sqrtf(sb / (float)W + eps_pair);
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const int i = (threadIdx.x + e * blockDim.x) * 4;
      if (i < W) {
        float xa[4], xb[4];
        Na4<float>::load(wa + i, xa);
        Na4<float>::load(wb + i, xb);
#pragma unroll
        for (int j = 0; j < 4; ++j) va[e][j] = va[e][j] * ia * xa[j] + vb[e][j] * ib * xb[j];
      }
    }
  }
  float s = 0.f;
#pragma unroll
  for (int e = 0; e < E; ++e)
#pragma unroll
    for (int j = 0; j < 4; ++j) s = fmaf(va[e][j], va[e][j], s);
  s = wave_sum(s);
  if (lane == 0) red[2][wave] = s;
  __syncthreads();
  s = 0.f;
  for (int k = 0; k < n_waves; ++k) s += red[2][k];
  const float inv = 1.f / sqrtf(s / (float)W + eps);
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int i = (threadIdx.x + e * blockDim.x) * 4;
    if (i < W) {
      float r[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) r[j] = res[e][j] + va[e][j] * inv * w[e][j];
      Na4<float>::store(residual + n * W + i, r);
      if (out) Na4<T>::store(out + n * W + i, r);
    }
  }
}

// Whether lmsf_norm_add takes rows of W entries (a multiple of 4 that a workgroup holds in registers).
extern "C" int lmsf_norm_add_fits(int W) { return W > 0 && W % 4 == 0 && W <= 16384; }

// a, b (null: none) [n_rows, W] of ``dtype`` with row strides that are multiples of 4 entries; residual contiguous float32
// [n_rows, W]; out (null: none) contiguous [n_rows, W] of ``dtype``; the weights float32 [W]; every row 16-byte aligned
// (8 bytes for bfloat16).
extern "C" int lmsf_norm_add(const void* a, long a_stride, const void* b, long b_stride, int dtype, const float* wa,
                             const float* wb, float eps_pair, float scale, const float* wn, float eps, float* residual,
                             void* out, int n_rows, int W, hipStream_t stream) {
  LMSF_CHECK(a && wn && residual && (!b || (wa && wb)), "norm_add: null pointer");
  LMSF_CHECK(dtype == LMSF_F32 || dtype == LMSF_BF16, "norm_add: unknown dtype code %d", dtype);
  LMSF_CHECK(lmsf_norm_add_fits(W) && a_stride >= W && (!b || b_stride >= W) && a_stride % 4 == 0 && b_stride % 4 == 0,
             "norm_add: rows of %d entries (multiples of 4 up to 16,384) at strides of multiples of 4", W);
  LMSF_CHECK(lmsf_aligned16(a) && (!b || lmsf_aligned16(b)) && lmsf_aligned16(residual) && lmsf_aligned16(wn) &&
                 (!out || lmsf_aligned16(out)) && (!b || (lmsf_aligned16(wa) && lmsf_aligned16(wb))),
             "norm_add: operands must be 16-byte aligned");
  if (n_rows <= 0) return 0;
  // many rows: small workgroups with several accesses a thread; few rows: as many threads as a row has groups of four
  const int quads = W / 4, per_thread = n_rows >= 512 ? 2 : 1;
  int threads = 64;
  while (threads < 1024 && threads * per_thread < quads) threads *= 2;
  const int need = (quads + threads - 1) / threads;
#define NA(T, P, E)                                                                                                  \
  hipLaunchKernelGGL((norm_add_kernel<T, P, E>), dim3(n_rows), dim3(threads), 0, stream, (const T*)a, a_stride,      \
                     (const T*)b, b_stride, wa, wb, eps_pair, scale, wn, eps, residual, (T*)out, W)
#define NA_E(T, P)               \
  do {                           \
    if (need <= 1) NA(T, P, 1);  \
    else if (need <= 2) NA(T, P, 2); \
    else NA(T, P, 4);            \
  } while (0)
  if (dtype == LMSF_F32) {
    if (b) NA_E(float, true); else NA_E(float, false);
  } else {
    if (b) NA_E(bf16_t, true); else NA_E(bf16_t, false);
  }
#undef NA_E
#undef NA
  LMSF_LAUNCH_CHECK("norm_add");
  return 0;
}
