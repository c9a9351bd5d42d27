// A real-gated linear recurrence (RG-LRU): one number of state per channel and request. The C channels are cut into
// equal blocks of c; with one square matrix [out, in] a block and gate, per token
//   r = sigmoid(Wr u + br),  i = sigmoid(Wi u + bi),  log a = -rate * r,
//   S <- a S + sqrt(1 - a^2) i u,   out = S * gelu_tanh(y)
// (rate = a constant times softplus of a weight, one number a channel, worked out when the weights are loaded). The
// reference has no recurrent mixer (its only one is attention over a paged cache,
// core/src/model_executor/layers/attention.rs:91-231).
//
//   lmsf_linear_recurrence_gates   a and b = sqrt(1 - a^2) i u of every token, float32 [N, C] each: both gates' products
//                                  in one launch (bfloat16, c a multiple of 32: on the matrix cores)
//   lmsf_linear_recurrence_scan    S and out from a and b. A segment of up to ``chunk`` tokens is walked by a thread a
//                                  channel, the state from the slot and back; a longer one (a prompt's portion) is cut
//                                  into chunks that run side by side: S is linear in the state it begins with, over a
//                                  chunk S_end = (prod a) S_begin + L, L the end that the chunk reaches from zero. One
//                                  launch leaves every chunk's (prod a, L), a small one folds them into every chunk's
//                                  S_begin, the last walks the chunks.
//   lmsf_linear_recurrence_step    a step of single tokens in one launch: the gates' products with the recurrence as
//                                  their epilogue.
//
// Segments, slots and the state's rows are as in recurrent.hip. 1 - a^2 is -expm1(2 log a), which keeps its digits where
// a is close to 1. All arithmetic is float32; results are rounded once, as stored.
#include "common.h"
#include "entry_points.h"

#include <math.h>

// In a float32 run the library's functions; in a bfloat16 run the hardware's 2^x, reciprocal and square root (float32 all
// the same, each good to the last bit or two: with the library's functions the gates' kernel took twice as long), and
// 1 - a^2 = -(e^x - 1), x = 2 log a, by the exponential's series where |x| < 1/2 and from a elsewhere.
template <typename T> struct LruMath;
template <> struct LruMath<float> {
  static __device__ __forceinline__ float sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
  static __device__ __forceinline__ float exp(float x) { return expf(x); }
  static __device__ __forceinline__ float root_rest(float log_a, float) { return sqrtf(fmaxf(-expm1f(2.f * log_a), 0.f)); }
};
template <> struct LruMath<bf16_t> {
  static __device__ __forceinline__ float sigmoid(float z) { return __builtin_amdgcn_rcpf(1.f + __expf(-z)); }
  static __device__ __forceinline__ float exp(float x) { return __expf(x); }
  static __device__ __forceinline__ float root_rest(float log_a, float a) {
    const float x = 2.f * log_a;
    float p = fmaf(x, 1.f / 40320.f, 1.f / 5040.f);
    p = fmaf(x, p, 1.f / 720.f);
    p = fmaf(x, p, 1.f / 120.f);
    p = fmaf(x, p, 1.f / 24.f);
    p = fmaf(x, p, 1.f / 6.f);
    p = fmaf(x, p, 0.5f);
    p = fmaf(x, p, 1.f);
    const float rest = x > -0.5f ? -x * p : fmaf(-a, a, 1.f);
    return __builtin_amdgcn_sqrtf(fmaxf(rest, 0.f));
  }
};

// the two gates' pre-activations and the channel's input -> a and b
template <typename T>
__device__ __forceinline__ void lru_coefficients(float r_pre, float i_pre, float u, float rate, float* a, float* b) {
  const float log_a = -rate * LruMath<T>::sigmoid(r_pre);
  *a = LruMath<T>::exp(log_a);
  *b = LruMath<T>::root_rest(log_a, *a) * LruMath<T>::sigmoid(i_pre) * u;
}

// Where the coefficients of (token t, channel ch) go: to memory, or (SINGLE) through the token's own state.
template <typename T>
struct LruOut {
  float* a;                     // [N, C] (gates)
  float* b;
  const T* y;                   // (step)
  long y_stride;
  float* state;
  long state_stride;
  const int* seg_of;
  const int* slots;
  T* out;
  long out_stride;
};
template <typename T, bool SINGLE>
__device__ __forceinline__ void lru_store(const LruOut<T>& o, int t, int C, int ch, float* st_row, float a, float b) {
  if constexpr (SINGLE) {
    const float S = fmaf(a, st_row[ch], b);
    st_row[ch] = S;
    o.out[(long)t * o.out_stride + ch] = from_f32<T>(S * gated_product_activation<5>(to_f32<T>(o.y[(long)t * o.y_stride + ch])));
  } else {
    o.a[(long)t * C + ch] = a;
    o.b[(long)t * C + ch] = b;
  }
}

// Any size, either type: a workgroup takes LRU_TOKENS tokens of one block, their inputs in LDS as float32; a thread owns
// outputs o, o + 256, ... and reads a row of each matrix once for all of them.
#define LRU_TOKENS 4
template <typename T, bool SINGLE>
__global__ __launch_bounds__(256) void lru_gates_kernel(const T* __restrict__ u, long u_stride, const T* __restrict__ Wr,
                                                        const float* __restrict__ br, const T* __restrict__ Wi,
                                                        const float* __restrict__ bi, const float* __restrict__ rate,
                                                        LruOut<T> o, int n_tokens, int C, int c) {
  extern __shared__ float su[];   // [LRU_TOKENS, c]
  const int blk = blockIdx.y, n0 = blockIdx.x * LRU_TOKENS, nt = min(LRU_TOKENS, n_tokens - n0);
  for (int i = threadIdx.x; i < LRU_TOKENS * c; i += 256) {
    const int t = i / c, k = i - t * c;
    su[i] = t < nt ? to_f32<T>(u[(long)(n0 + t) * u_stride + (long)blk * c + k]) : 0.f;
  }
  __syncthreads();
  for (int j = blockIdx.z * 256 + threadIdx.x; j < c; j += gridDim.z * 256) {
    const T* rr = Wr + ((long)blk * c + j) * c;
    const T* ri = Wi + ((long)blk * c + j) * c;
    float ar[LRU_TOKENS], ai[LRU_TOKENS];
#pragma unroll
    for (int t = 0; t < LRU_TOKENS; ++t) ar[t] = ai[t] = 0.f;
    for (int k = 0; k < c; ++k) {
      const float wr = to_f32<T>(rr[k]), wi = to_f32<T>(ri[k]);
#pragma unroll
      for (int t = 0; t < LRU_TOKENS; ++t) {
        ar[t] = fmaf(wr, su[t * c + k], ar[t]);
        ai[t] = fmaf(wi, su[t * c + k], ai[t]);
      }
    }
    const int ch = blk * c + j;
#pragma unroll
    for (int t = 0; t < LRU_TOKENS; ++t)
      if (t < nt) {
        float a, b;
        lru_coefficients<T>(ar[t] + br[ch], ai[t] + bi[ch], su[t * c + j], rate[ch], &a, &b);
        float* st = SINGLE ? o.state + (long)o.slots[o.seg_of[n0 + t]] * o.state_stride : nullptr;
        lru_store<T, SINGLE>(o, n0 + t, C, ch, st, a, b);
      }
  }
}

// The same on the matrix cores (bfloat16, c a multiple of 32, rows and blocks at multiples of 16 bytes): a wave takes 16
// outputs of a block (A: 16 rows of each gate's matrix x 32 k) and MT tiles of 16 tokens (B), both gates' products from
// the same fragments of u.
template <int MT, bool SINGLE>
__global__ __launch_bounds__(256) void lru_gates_mfma_kernel(const bf16_t* __restrict__ u, long u_stride,
                                                             const bf16_t* __restrict__ Wr, const float* __restrict__ br,
                                                             const bf16_t* __restrict__ Wi, const float* __restrict__ bi,
                                                             const float* __restrict__ rate, LruOut<bf16_t> o,
                                                             int n_tokens, int C, int c) {
  const int blk = blockIdx.y, n0 = blockIdx.x * (16 * MT);
  const int wave = threadIdx.x / LMSF_WAVE, lane = threadIdx.x % LMSF_WAVE;
  const int fr = lane % 16, fg = lane / 16;
  const int j0 = (blockIdx.z * (blockDim.x / LMSF_WAVE) + wave) * 16;
  if (j0 >= c) return;
  const long w_at = ((long)blk * c + min(j0 + fr, c - 1)) * c + fg * 8;
  const bf16_t* xb[MT];
  int tok[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    tok[mt] = n0 + mt * 16 + fr;
    xb[mt] = u + (long)min(tok[mt], n_tokens - 1) * u_stride + (long)blk * c;
  }
  f32x4_t ar[MT], ai[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) ar[mt] = ai[mt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int k = 0; k < c; k += 32) {
    const bf16x8_t fwr = *reinterpret_cast<const bf16x8_t*>(Wr + w_at + k);
    const bf16x8_t fwi = *reinterpret_cast<const bf16x8_t*>(Wi + w_at + k);
    bf16x8_t fb[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) fb[mt] = *reinterpret_cast<const bf16x8_t*>(xb[mt] + k + fg * 8);
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      ar[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fwr, fb[mt], ar[mt], 0, 0, 0);
      ai[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fwi, fb[mt], ai[mt], 0, 0, 0);
    }
  }
  // lane: token fr of every tile, outputs j0 + fg * 4 .. + 3 (c is a multiple of 16: all of them or none)
  const int jl = j0 + fg * 4, ch0 = blk * c + jl;
  const float4 vbr = *reinterpret_cast<const float4*>(br + ch0), vbi = *reinterpret_cast<const float4*>(bi + ch0);
  const float4 vra = *reinterpret_cast<const float4*>(rate + ch0);
  const float brv[4] = {vbr.x, vbr.y, vbr.z, vbr.w}, biv[4] = {vbi.x, vbi.y, vbi.z, vbi.w};
  const float rav[4] = {vra.x, vra.y, vra.z, vra.w};
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    if (tok[mt] >= n_tokens) continue;
    const uint2 uw = *reinterpret_cast<const uint2*>(xb[mt] + jl);
    const float uv[4] = {__uint_as_float(uw.x << 16), __uint_as_float(uw.x & 0xffff0000u), __uint_as_float(uw.y << 16),
                         __uint_as_float(uw.y & 0xffff0000u)};
    float a[4], b[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) lru_coefficients<bf16_t>(ar[mt][j] + brv[j], ai[mt][j] + biv[j], uv[j], rav[j], &a[j], &b[j]);
    if constexpr (SINGLE) {
      float* st = o.state + (long)o.slots[o.seg_of[tok[mt]]] * o.state_stride;
#pragma unroll
      for (int j = 0; j < 4; ++j) lru_store<bf16_t, true>(o, tok[mt], C, ch0 + j, st, a[j], b[j]);
    } else {
      *reinterpret_cast<float4*>(o.a + (long)tok[mt] * C + ch0) = make_float4(a[0], a[1], a[2], a[3]);
      *reinterpret_cast<float4*>(o.b + (long)tok[mt] * C + ch0) = make_float4(b[0], b[1], b[2], b[3]);
    }
  }
}

// For many tokens: the workgroup's 16 MT tokens of the block lie in LDS, read once from memory and by all its waves; wave
// w takes the outputs 16 w, 16 (w + WAVES), ... of the block. (With every wave fetching u for itself 30 us at
// 2,048 tokens of 2,048 channels in blocks of 256.)
#define LRU_PAD 8             // entries between rows in LDS, so that the 16 rows of a fragment lie in different banks
template <int MT, int WAVES>
__global__ __launch_bounds__(WAVES * LMSF_WAVE) void lru_gates_tile_kernel(
    const bf16_t* __restrict__ u, long u_stride, const bf16_t* __restrict__ Wr, const float* __restrict__ br,
    const bf16_t* __restrict__ Wi, const float* __restrict__ bi, const float* __restrict__ rate, float* __restrict__ a_out,
    float* __restrict__ b_out, int n_tokens, int C, int c) {
  extern __shared__ __align__(16) bf16_t tile[];        // [16 MT][c + LRU_PAD]
  const int blk = blockIdx.y, n0 = blockIdx.x * (16 * MT), ld = c + LRU_PAD;
  const int wave = threadIdx.x / LMSF_WAVE, lane = threadIdx.x % LMSF_WAVE, fr = lane % 16, fg = lane / 16;
  const int per_row = c / 8;
  for (int i = threadIdx.x; i < 16 * MT * per_row; i += WAVES * LMSF_WAVE) {
    const int t = i / per_row, k = (i - t * per_row) * 8;
    *reinterpret_cast<uint4*>(tile + t * ld + k) =
        *reinterpret_cast<const uint4*>(u + (long)min(n0 + t, n_tokens - 1) * u_stride + (long)blk * c + k);
  }
  __syncthreads();
  for (int j0 = wave * 16; j0 < c; j0 += WAVES * 16) {
    const long w_at = ((long)blk * c + j0 + fr) * c + fg * 8;
    f32x4_t ar[MT], ai[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) ar[mt] = ai[mt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k = 0; k < c; k += 32) {
      const bf16x8_t fwr = *reinterpret_cast<const bf16x8_t*>(Wr + w_at + k);
      const bf16x8_t fwi = *reinterpret_cast<const bf16x8_t*>(Wi + w_at + k);
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        const bf16x8_t fb = *reinterpret_cast<const bf16x8_t*>(tile + (mt * 16 + fr) * ld + k + fg * 8);
        ar[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fwr, fb, ar[mt], 0, 0, 0);
        ai[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fwi, fb, ai[mt], 0, 0, 0);
      }
    }
    const int jl = j0 + fg * 4, ch0 = blk * c + jl;
    const float4 vbr = *reinterpret_cast<const float4*>(br + ch0), vbi = *reinterpret_cast<const float4*>(bi + ch0);
    const float4 vra = *reinterpret_cast<const float4*>(rate + ch0);
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      const int t = n0 + mt * 16 + fr;
      if (t >= n_tokens) continue;
      const uint2 uw = *reinterpret_cast<const uint2*>(tile + (mt * 16 + fr) * ld + jl);
      float4 a, b;
      lru_coefficients<bf16_t>(ar[mt][0] + vbr.x, ai[mt][0] + vbi.x, __uint_as_float(uw.x << 16), vra.x, &a.x, &b.x);
      lru_coefficients<bf16_t>(ar[mt][1] + vbr.y, ai[mt][1] + vbi.y, __uint_as_float(uw.x & 0xffff0000u), vra.y, &a.y, &b.y);
      lru_coefficients<bf16_t>(ar[mt][2] + vbr.z, ai[mt][2] + vbi.z, __uint_as_float(uw.y << 16), vra.z, &a.z, &b.z);
      lru_coefficients<bf16_t>(ar[mt][3] + vbr.w, ai[mt][3] + vbi.w, __uint_as_float(uw.y & 0xffff0000u), vra.w, &a.w, &b.w);
      *reinterpret_cast<float4*>(a_out + (long)t * C + ch0) = a;
      *reinterpret_cast<float4*>(b_out + (long)t * C + ch0) = b;
    }
  }
}

// ---------------------------------------------------------------- the scan

#define LRU_TT 8          // tokens whose operands a thread asks for together

template <typename T, bool SUMMARY>
__global__ __launch_bounds__(256) void lru_scan_kernel(const float* __restrict__ a, const float* __restrict__ b,
                                                       const T* __restrict__ y, long y_stride, float* __restrict__ state,
                                                       long state_stride, const int* __restrict__ seg_starts,
                                                       const int* __restrict__ slots, T* __restrict__ out,
                                                       long out_stride, int C, int chunk,
                                                       const int* __restrict__ scratch_base, float* __restrict__ scratch) {
  const int ch = blockIdx.x * 256 + threadIdx.x;
  const int s = blockIdx.z, j = blockIdx.y;
  const int seg_start = seg_starts[s], seg_end = seg_starts[s + 1];
  const int base = scratch_base ? scratch_base[s] : -1;
  if (ch >= C || (SUMMARY && base < 0)) return;
  const int n_chunks = base < 0 ? 1 : (seg_end - seg_start + chunk - 1) / chunk;
  if (j >= n_chunks || seg_end <= seg_start) return;
  const int start = base < 0 ? seg_start : seg_start + j * chunk;
  const int end = base < 0 ? seg_end : min(seg_end, start + chunk);
  const long entry = 2L * C;                      // S at the chunk's beginning (before the fold: L of the chunk before), prod a
  float* st = state + (long)slots[s] * state_stride + ch;
  float S = 0.f, prod = 1.f;
  if (SUMMARY) {
    if (j == 0) scratch[(long)base * entry + ch] = *st;                  // the entry before the first chunk
    if (j == n_chunks - 1) return;                                       // nobody folds the last chunk's summary
  } else {
    S = base < 0 ? *st : scratch[(long)(base + j) * entry + ch];
  }
  for (int t0 = start; t0 < end; t0 += LRU_TT) {
    const int nt = min(LRU_TT, end - t0);
    float va[LRU_TT], vb[LRU_TT], vy[LRU_TT];
#pragma unroll
    for (int i = 0; i < LRU_TT; ++i) {
      const long t = t0 + (i < nt ? i : 0);
      va[i] = a[t * C + ch];
      vb[i] = b[t * C + ch];
      vy[i] = SUMMARY ? 0.f : to_f32<T>(y[t * y_stride + ch]);
    }
#pragma unroll
    for (int i = 0; i < LRU_TT; ++i) {
      if (i < nt) {
        S = fmaf(va[i], S, vb[i]);
        if (SUMMARY) prod *= va[i];
        else out[(long)(t0 + i) * out_stride + ch] = from_f32<T>(S * gated_product_activation<5>(vy[i]));
      }
    }
  }
  if (SUMMARY) {
    float* ent = scratch + (long)(base + j + 1) * entry;
    ent[ch] = S;
    ent[C + ch] = prod;
  } else if (j == n_chunks - 1) {
    *st = S;
  }
}

// Between the two: entry e > 0 holds chunk e - 1's (L, prod a); afterwards the state at the beginning of chunk e.
__global__ __launch_bounds__(64) void lru_fold_kernel(const int* __restrict__ seg_starts, const int* __restrict__ scratch_base,
                                                      float* __restrict__ scratch, int C, int chunk) {
  const int s = blockIdx.y, base = scratch_base[s];
  const int ch = blockIdx.x * 64 + threadIdx.x;
  if (base < 0 || ch >= C) return;
  const int n_chunks = (seg_starts[s + 1] - seg_starts[s] + chunk - 1) / chunk;
  const long entry = 2L * C;
  float* ent = scratch + (long)base * entry + ch;
  float S = ent[0];
  for (int e = 1; e < n_chunks; e += LRU_TT) {
    float L[LRU_TT], p[LRU_TT];
#pragma unroll
    for (int i = 0; i < LRU_TT; ++i) {
      const long at = (long)min(e + i, n_chunks - 1) * entry;
      L[i] = ent[at];
      p[i] = ent[at + C];
    }
#pragma unroll
    for (int i = 0; i < LRU_TT; ++i)
      if (e + i < n_chunks) {
        S = fmaf(p[i], S, L[i]);
        ent[(long)(e + i) * entry] = S;
      }
  }
}

// floats of scratch a chunk takes
extern "C" long lmsf_linear_recurrence_entry_floats(int C) { return 2L * C; }

#define LRU_TILE_MIN_TOKENS 256
template <typename T, bool SINGLE>
static void launch_gates(const void* u, int dtype, long u_stride, const void* Wr, const float* br, const void* Wi,
                         const float* bi, const float* rate, const LruOut<T>& o, int n_tokens, int C, int c,
                         hipStream_t stream) {
  const int blocks = C / c;
  if constexpr (sizeof(T) == 2) {
    if (c % 32 == 0 && u_stride % 8 == 0 && lmsf_aligned16(u) && lmsf_aligned16(Wr) && lmsf_aligned16(Wi) &&
        lmsf_aligned16(br) && lmsf_aligned16(bi) && lmsf_aligned16(rate) && (SINGLE || (lmsf_aligned16(o.a) && lmsf_aligned16(o.b)))) {
      if constexpr (!SINGLE) {
#define LRU_TILE(MT)                                                                                                \
  hipLaunchKernelGGL((lru_gates_tile_kernel<MT, 8>), dim3((n_tokens + 16 * MT - 1) / (16 * MT), blocks),             \
                     dim3(8 * LMSF_WAVE), (size_t)16 * MT * (c + LRU_PAD) * 2, stream, (const bf16_t*)u, u_stride,   \
                     (const bf16_t*)Wr, br, (const bf16_t*)Wi, bi, rate, o.a, o.b, n_tokens, C, c)
        // 64 tokens a workgroup where that still fills the chip (the matrices are read once a workgroup: 2,048 tokens of
        // 2,048 channels in blocks of 256 20 us against 25 with 32 tokens and 38 with 16), else 32
        const size_t row = (size_t)(c + LRU_PAD) * 2;
        if (n_tokens >= LRU_TILE_MIN_TOKENS && 64 * row <= 64 * 1024 && (long)((n_tokens + 63) / 64) * blocks >= lmsf_compute_units()) {
          LRU_TILE(4);
          return;
        }
        if (n_tokens >= LRU_TILE_MIN_TOKENS && 32 * row <= 64 * 1024) {
          LRU_TILE(2);
          return;
        }
#undef LRU_TILE
      }
      // few tokens: a wave a workgroup, so that the matrices' rows are read by as many compute units as there are
#define LRU_MFMA(MT, W)                                                                                             \
  hipLaunchKernelGGL((lru_gates_mfma_kernel<MT, SINGLE>), dim3((n_tokens + 16 * MT - 1) / (16 * MT), blocks,        \
                                                               (c + 16 * W - 1) / (16 * W)),                         \
                     dim3(64 * W), 0, stream, (const bf16_t*)u, u_stride, (const bf16_t*)Wr, br, (const bf16_t*)Wi, \
                     bi, rate, o, n_tokens, C, c)
      if (n_tokens <= 64) LRU_MFMA(1, 1);
      else if ((long)((n_tokens + 63) / 64) * blocks * ((c + 63) / 64) < 512) LRU_MFMA(1, 4);
      else LRU_MFMA(4, 4);
#undef LRU_MFMA
      return;
    }
  }
  const dim3 grid((n_tokens + LRU_TOKENS - 1) / LRU_TOKENS, blocks, (c + 255) / 256);
  hipLaunchKernelGGL((lru_gates_kernel<T, SINGLE>), grid, dim3(256), (size_t)LRU_TOKENS * c * 4, stream, (const T*)u,
                     u_stride, (const T*)Wr, br, (const T*)Wi, bi, rate, o, n_tokens, C, c);
}

static int check_gates(const char* who, const void* u, int dtype, long u_stride, const void* Wr, const float* br,
                       const void* Wi, const float* bi, const float* rate, int C, int c) {
  LMSF_CHECK(u && Wr && br && Wi && bi && rate, "%s: null pointer", who);
  LMSF_CHECK(dtype == LMSF_F32 || dtype == LMSF_BF16, "%s: unknown dtype code %d", who, dtype);
  LMSF_CHECK(C > 0 && c > 0 && C % c == 0 && C / c <= 65535 && u_stride >= C, "%s: bad sizes C=%d c=%d", who, C, c);
  LMSF_CHECK((size_t)LRU_TOKENS * c * 4 <= 64 * 1024, "%s: blocks of %d channels do not fit LDS (at most %d)", who, c,
             64 * 1024 / (LRU_TOKENS * 4));
  return 0;
}

// u [N, C] of ``dtype``, Wr, Wi [C / c, c, c] of ``dtype``, br, bi, rate float32 [C] -> a, b float32 [N, C]
extern "C" int lmsf_linear_recurrence_gates(const void* u, int dtype, long u_stride, const void* Wr, const float* br,
                                            const void* Wi, const float* bi, const float* rate, float* a, float* b,
                                            int n_tokens, int C, int c, hipStream_t stream) {
  if (int rc = check_gates("linear_recurrence_gates", u, dtype, u_stride, Wr, br, Wi, bi, rate, C, c)) return rc;
  LMSF_CHECK(a && b, "linear_recurrence_gates: null pointer");
  if (n_tokens <= 0) return 0;
  if (dtype == LMSF_F32) {
    const LruOut<float> o = {a, b, nullptr, 0, nullptr, 0, nullptr, nullptr, nullptr, 0};
    launch_gates<float, false>(u, dtype, u_stride, Wr, br, Wi, bi, rate, o, n_tokens, C, c, stream);
  } else {
    const LruOut<bf16_t> o = {a, b, nullptr, 0, nullptr, 0, nullptr, nullptr, nullptr, 0};
    launch_gates<bf16_t, false>(u, dtype, u_stride, Wr, br, Wi, bi, rate, o, n_tokens, C, c, stream);
  }
  LMSF_LAUNCH_CHECK("linear_recurrence_gates");
  return 0;
}

// A step in which every token is its request's only one: gates, recurrence and the product with gelu_tanh(y) together.
// state float32 [slots, >= C]; out [N, C] of ``dtype``.
extern "C" int lmsf_linear_recurrence_step(const void* u, int dtype, long u_stride, const void* Wr, const float* br,
                                           const void* Wi, const float* bi, const float* rate, const void* y,
                                           long y_stride, float* state, long state_stride, const int* seg_of,
                                           const int* slots, void* out, long out_stride, int n_tokens, int C, int c,
                                           hipStream_t stream) {
  if (int rc = check_gates("linear_recurrence_step", u, dtype, u_stride, Wr, br, Wi, bi, rate, C, c)) return rc;
  LMSF_CHECK(y && state && seg_of && slots && out, "linear_recurrence_step: null pointer");
  LMSF_CHECK(y_stride >= C && state_stride >= C && out_stride >= C, "linear_recurrence_step: strides too small");
  if (n_tokens <= 0) return 0;
  if (dtype == LMSF_F32) {
    const LruOut<float> o = {nullptr, nullptr, (const float*)y, y_stride, state, state_stride, seg_of, slots, (float*)out, out_stride};
    launch_gates<float, true>(u, dtype, u_stride, Wr, br, Wi, bi, rate, o, n_tokens, C, c, stream);
  } else {
    const LruOut<bf16_t> o = {nullptr, nullptr, (const bf16_t*)y, y_stride, state, state_stride, seg_of, slots, (bf16_t*)out, out_stride};
    launch_gates<bf16_t, true>(u, dtype, u_stride, Wr, br, Wi, bi, rate, o, n_tokens, C, c, stream);
  }
  LMSF_LAUNCH_CHECK("linear_recurrence_step");
  return 0;
}

// ``scratch_base``, ``scratch``: segments with a non-negative base are cut into chunks of ``chunk`` tokens
// (``max_chunks``: the most chunks any of them has) whose entries begin there; null: every segment is one chunk.
extern "C" int lmsf_linear_recurrence_scan(const float* a, const float* b, const void* y, int dtype, long y_stride,
                                           float* state, long state_stride, const int* seg_starts, const int* slots,
                                           void* out, long out_stride, int n_tokens, int n_segments, int C, int chunk,
                                           int max_chunks, const int* scratch_base, float* scratch,
                                           hipStream_t stream) {
  LMSF_CHECK(a && b && y && state && seg_starts && slots && out, "linear_recurrence_scan: null pointer");
  LMSF_CHECK(dtype == LMSF_F32 || dtype == LMSF_BF16, "linear_recurrence_scan: unknown dtype code %d", dtype);
  LMSF_CHECK(C > 0 && y_stride >= C && state_stride >= C && out_stride >= C, "linear_recurrence_scan: strides too small");
  LMSF_CHECK(n_tokens >= 0 && n_segments >= 0 && n_segments <= 65535, "linear_recurrence_scan: bad counts");
  const bool chunked = scratch_base != nullptr;
  LMSF_CHECK(!chunked || (scratch && chunk > 0 && max_chunks >= 1 && max_chunks <= 65535),
             "linear_recurrence_scan: the chunked form needs scratch, a chunk size and the number of chunks");
  if (n_tokens == 0 || n_segments == 0) return 0;
  const dim3 grid((C + 255) / 256, chunked ? max_chunks : 1, n_segments), block(256);
#define LRU_SCAN(T, SUM)                                                                                              \
  hipLaunchKernelGGL((lru_scan_kernel<T, SUM>), grid, block, 0, stream, a, b, (const T*)y, y_stride, state,           \
                     state_stride, seg_starts, slots, (T*)out, out_stride, C, chunk, scratch_base, scratch)
  if (chunked) {
    if (dtype == LMSF_F32) LRU_SCAN(float, true); else LRU_SCAN(bf16_t, true);
    LMSF_LAUNCH_CHECK("linear_recurrence_scan (chunk summaries)");
    hipLaunchKernelGGL(lru_fold_kernel, dim3((C + 63) / 64, n_segments), dim3(64), 0, stream, seg_starts, scratch_base,
                       scratch, C, chunk);
    LMSF_LAUNCH_CHECK("linear_recurrence_scan (fold)");
  }
  if (dtype == LMSF_F32) LRU_SCAN(float, false); else LRU_SCAN(bf16_t, false);
#undef LRU_SCAN
  LMSF_LAUNCH_CHECK("linear_recurrence_scan");
  return 0;
}
