// A linear recurrence with one decay a head and a state of N x dv numbers a head (Mamba-2's). Per head h, with B and C of
// its group h / (H / G), dt = softplus(dt_pre + dt_bias), and rate = exp(A_log):
//     S_t = exp(-rate dt) S_(t-1) + dt B_t x_t^T,     y_t = S_t^T C_t + D x_t
// x, B and C are columns of one buffer as the short convolution left them; dt_pre, the decays, the state and y are float32.
// The state of a slot is [H, dv, N] float32 (for every head the N numbers of a value entry side by side), all zeros when
// a request begins. The reference has no such mixer (its only one is attention over a paged cache,
// core/src/model_executor/layers/attention.rs:91-231).
//
// Two forms:
// - token by token, the state in registers over a segment's tokens: 4 to 64 lanes hold a value entry's N numbers, four
//   neighbours each (or several times four). Steps of single tokens stream the state once; float32 runs and sizes that the
//   other form does not take run it too.
// - chunks of 64 tokens side by side on the matrix cores (bfloat16 runs). With c_t the sum of the logarithms of the decays
//   from the chunk's start to t, S_0 the state before the chunk, L its last token:
//       y_t = exp(c_t) S_0^T C_t + sum_{u<=t} exp(c_t - c_u) dt_u (C_t . B_u) x_u + D x_t
//       U   = sum_u exp(c_L - c_u) dt_u B_u x_u^T,      S_L = exp(c_L) S_0 + U
//   in three launches: U of every chunk, a fold over a segment's chunks (S_0 takes U's place), the outputs. B, C and x are
//   bfloat16 numbers; whatever is float32 beside them in a product (S_0, the decayed and stepped C . B, x times its step)
//   enters as three bfloat16 parts whose sum it is exactly, so the products are float32 products. Sums of logarithms are
//   carried as two floats (from a float64 prefix sum), so that a difference of two of them is good to its own last bit.
#include "common.h"
#include "entry_points.h"

#include <math.h>

#define SS_L 64              // tokens of a chunk
#define SS_MAX_STATE 1024    // N
#define SS_PT (4 * 2 * 3 * 64 * 16)   // bytes of a chunk's decayed C . B in parts

__device__ __forceinline__ float ss_softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }

extern "C" long lmsf_state_space_state_floats(int H, int N, int dv) { return (long)H * N * dv; }

// ---------------------------------------------------------------- token by token

__device__ __forceinline__ void ss_load4(const float* p, float* x) {
  const float4 v = *reinterpret_cast<const float4*>(p);
  x[0] = v.x, x[1] = v.y, x[2] = v.z, x[3] = v.w;
}
__device__ __forceinline__ void ss_load4(const bf16_t* p, float* x) {
  const uint2 v = *reinterpret_cast<const uint2*>(p);
  x[0] = __uint_as_float(v.x << 16), x[1] = __uint_as_float(v.x & 0xffff0000u);
  x[2] = __uint_as_float(v.y << 16), x[3] = __uint_as_float(v.y & 0xffff0000u);
}
__device__ __forceinline__ void ss_store4(float* p, const float* x) {
  *reinterpret_cast<float4*>(p) = make_float4(x[0], x[1], x[2], x[3]);
}
__device__ __forceinline__ void ss_store4(bf16_t* p, const float* x) {
  *reinterpret_cast<uint2*>(p) = make_uint2(pack2_bf16(x[0], x[1]), pack2_bf16(x[2], x[3]));
}
// four neighbours from entry n of n_all on (VEC: whole groups at aligned places; else entries beyond the end are zeros)
template <bool VEC, typename T>
__device__ __forceinline__ void ss_get4(const T* __restrict__ p, int n, int n_all, float* x) {
  if (VEC) {
    if (n < n_all) ss_load4(p + n, x);
    else x[0] = x[1] = x[2] = x[3] = 0.f;
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j) x[j] = n + j < n_all ? to_f32<T>(p[n + j]) : 0.f;
  }
}

// LPR lanes hold a value entry's numbers, K groups of four each; R value entries a group of lanes
template <typename T, int LPR, int K, int R, bool VEC>
__global__ __launch_bounds__(256) void state_space_token_kernel(
    const T* __restrict__ xbc, long xbc_stride, int x_at, int b_at, int c_at, const float* __restrict__ dt_pre,
    long dt_stride, const float* __restrict__ dt_bias, const float* __restrict__ rate, const float* __restrict__ D,
    float* __restrict__ state, long state_stride, const int* __restrict__ seg_starts,
    const int* __restrict__ state_slots, float* __restrict__ y, long y_stride, int H, int G, int N, int dv) {
  constexpr int GROUPS = 256 / LPR;
  const int h = blockIdx.y, s = blockIdx.z, g = h / (H / G);
  const int lr = threadIdx.x % LPR, grp = threadIdx.x / LPR;
  const int e0 = blockIdx.x * GROUPS * R + grp;
  float* S = state + (long)state_slots[s] * state_stride + (long)h * dv * N;
  const float bias = dt_bias[h], rt = rate[h], skip = D[h];
  float st[R][K][4];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int e = e0 + r * GROUPS;
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int n = (k * LPR + lr) * 4;
      if (e < dv) ss_get4<VEC, float>(S + (long)e * N, n, N, st[r][k]);
      else st[r][k][0] = st[r][k][1] = st[r][k][2] = st[r][k][3] = 0.f;
    }
  }
  const int t1 = seg_starts[s + 1];
  for (int t = seg_starts[s]; t < t1; ++t) {
    const T* row = xbc + (long)t * xbc_stride;
    float bv[K][4], cv[K][4], xv[R], acc[R];
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int n = (k * LPR + lr) * 4;
      ss_get4<VEC, T>(row + b_at + g * N, n, N, bv[k]);
      ss_get4<VEC, T>(row + c_at + g * N, n, N, cv[k]);
    }
#pragma unroll
    for (int r = 0; r < R; ++r) xv[r] = to_f32<T>(row[x_at + h * dv + min(e0 + r * GROUPS, dv - 1)]);
    const float dt = ss_softplus(dt_pre[(long)t * dt_stride + h] + bias);
    const float keep = expf(-rt * dt);
#pragma unroll
    for (int r = 0; r < R; ++r) {
      acc[r] = 0.f;
      const float dx = dt * xv[r];
#pragma unroll
      for (int k = 0; k < K; ++k)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          st[r][k][j] = fmaf(keep, st[r][k][j], bv[k][j] * dx);
          acc[r] = fmaf(st[r][k][j], cv[k][j], acc[r]);
        }
    }
#pragma unroll
    for (int o = LPR / 2; o > 0; o >>= 1)
#pragma unroll
      for (int r = 0; r < R; ++r) acc[r] += __shfl_xor(acc[r], o, LMSF_WAVE);
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const int e = e0 + r * GROUPS;
      if (lr == 0 && e < dv) y[(long)t * y_stride + (long)h * dv + e] = fmaf(skip, xv[r], acc[r]);
    }
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int e = e0 + r * GROUPS;
    if (e >= dv) continue;
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int n = (k * LPR + lr) * 4;
      float* p = S + (long)e * N + n;
      if (VEC) {
        if (n < N) *reinterpret_cast<float4*>(p) = make_float4(st[r][k][0], st[r][k][1], st[r][k][2], st[r][k][3]);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (n + j < N) p[j] = st[r][k][j];
      }
    }
  }
}

// ---------------------------------------------------------------- chunks

// a float32 number as three bfloat16 numbers whose sum it is; two numbers a call, packed
__device__ __forceinline__ void ss_parts2(float a, float b, uint32_t& p0, uint32_t& p1, uint32_t& p2) {
  p0 = pack2_bf16(a, b);
  const float ra = a - __uint_as_float(p0 << 16), rb = b - __uint_as_float(p0 & 0xffff0000u);
  p1 = pack2_bf16(ra, rb);
  p2 = pack2_bf16(ra - __uint_as_float(p1 << 16), rb - __uint_as_float(p1 & 0xffff0000u));
}
union SsFrag {
  bf16x8_t v;
  uint4 q;
  uint2 h[2];
  uint32_t w[4];
};
__device__ __forceinline__ void ss_parts8(const float* x, SsFrag (&f)[3]) {
#pragma unroll
  for (int i = 0; i < 4; ++i) ss_parts2(x[2 * i], x[2 * i + 1], f[0].w[i], f[1].w[i], f[2].w[i]);
}

// A chunk's matrix of bfloat16 [64 tokens][cols] turned, in LDS: row c holds the tokens 0 .. 63 in eight pieces of eight
// (16 bytes), piece p at place p ^ swizzle(c), so that neither the turned writes nor the reads of eight tokens of 16
// rows fall into the same banks.
__device__ __forceinline__ int ss_turned(int c, int piece) { return c * 128 + (((piece ^ c ^ (c >> 3)) & 7) << 4); }

// Columns [0, cols) of 64 rows (``src`` at the chunk's first token, ``nt`` tokens, the others zeros) turned into ``dst``
// [cols_padded][64]; ``vec``: whole groups of eight columns at aligned places. A thread takes two tokens of eight columns
// a time, and asks for two such pieces before it stores one.
__device__ __forceinline__ void ss_put_turned(const SsFrag& a, const SsFrag& b, int c0, int t, int cols_padded,
                                              unsigned char* dst) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const int c = c0 + j;
    if (c >= cols_padded) break;
    const uint32_t lo = (j & 1) ? a.w[j >> 1] >> 16 : a.w[j >> 1] & 0xffffu;
    const uint32_t hi = (j & 1) ? b.w[j >> 1] >> 16 : b.w[j >> 1] & 0xffffu;
    *reinterpret_cast<uint32_t*>(dst + ss_turned(c, t >> 3) + (t & 7) * 2) = lo | (hi << 16);
  }
}
__device__ __forceinline__ void ss_stage_turned(const bf16_t* __restrict__ src, long stride, int nt, int cols,
                                                int cols_padded, bool vec, unsigned char* dst) {
  const int blocks = (cols_padded + 7) / 8, items = blocks * (SS_L / 2);
  if (vec) {
    // (rows and columns outside are read from the last ones and dropped: no branch around a load)
    for (int i0 = threadIdx.x; i0 < items; i0 += 512) {
      SsFrag r[2][2];
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const int i = min(i0 + k * 256, items - 1), c0 = min((i % blocks) * 8, cols - 8), t = 2 * (i / blocks);
        r[k][0].q = *reinterpret_cast<const uint4*>(src + (long)min(t, nt - 1) * stride + c0);
        r[k][1].q = *reinterpret_cast<const uint4*>(src + (long)min(t + 1, nt - 1) * stride + c0);
      }
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const int i = i0 + k * 256, c0 = (i % blocks) * 8, t = 2 * (i / blocks);
        if (i >= items) break;
        if (c0 >= cols || t >= nt) r[k][0].q = make_uint4(0, 0, 0, 0);
        if (c0 >= cols || t + 1 >= nt) r[k][1].q = make_uint4(0, 0, 0, 0);
        ss_put_turned(r[k][0], r[k][1], c0, t, cols_padded, dst);
      }
    }
    return;
  }
  for (int i = threadIdx.x; i < items; i += 256) {
    const int c0 = (i % blocks) * 8, t = 2 * (i / blocks);
    SsFrag a, b;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      uint32_t x[4];
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int c = c0 + 2 * j + (q & 1), tt = t + (q >> 1);
        x[q] = c < cols && tt < nt ? src[(long)tt * stride + c] : 0;
      }
      a.w[j] = x[0] | (x[1] << 16);
      b.w[j] = x[2] | (x[3] << 16);
    }
    ss_put_turned(a, b, c0, t, cols_padded, dst);
  }
}

// Two matrices of the same columns as they lie (C and B), rows of ``row_bytes``, one behind the other from ``dst`` on
// (``apart`` bytes).
__device__ __forceinline__ void ss_stage_two(const bf16_t* __restrict__ src0, const bf16_t* __restrict__ src1, long stride,
                                             int nt, int cols, int cols_padded, bool vec, unsigned char* dst, int apart,
                                             int row_bytes) {
  const int blocks = cols_padded / 8, items = 2 * SS_L * blocks;
  if (vec) {
    for (int i0 = threadIdx.x; i0 < items; i0 += 8 * 256) {
      uint4 r[8];
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        const int i = min(i0 + k * 256, items - 1), row = i / blocks, c0 = min((i - row * blocks) * 8, cols - 8);
        const bf16_t* src = row < SS_L ? src0 : src1;
        r[k] = *reinterpret_cast<const uint4*>(src + (long)min(row & (SS_L - 1), nt - 1) * stride + c0);
      }
#pragma unroll
      for (int k = 0; k < 8; ++k) {
        const int i = i0 + k * 256, row = i / blocks, c0 = (i - row * blocks) * 8, t = row & (SS_L - 1);
        if (i >= items) break;
        if (c0 >= cols || t >= nt) r[k] = make_uint4(0, 0, 0, 0);
        *reinterpret_cast<uint4*>(dst + (row < SS_L ? 0 : apart) + t * row_bytes + c0 * 2) = r[k];
      }
    }
    return;
  }
  for (int i = threadIdx.x; i < items; i += 256) {
    const int row = i / blocks, c0 = (i - row * blocks) * 8, t = row & (SS_L - 1);
    const bf16_t* src = row < SS_L ? src0 : src1;
    SsFrag a;
    a.q = make_uint4(0, 0, 0, 0);
    if (t < nt) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int c = c0 + 2 * j;
        const uint32_t lo = c < cols ? src[(long)t * stride + c] : 0, hi = c + 1 < cols ? src[(long)t * stride + c + 1] : 0;
        a.w[j] = lo | (hi << 16);
      }
    }
    *reinterpret_cast<uint4*>(dst + (row < SS_L ? 0 : apart) + t * row_bytes + c0 * 2) = a.q;
  }
}

// The head of a workgroup: workgroups go to the eight dies in turn, and neighbouring heads (which share a group's B and C)
// are given to one die.
__device__ __forceinline__ int ss_head(int H) {
  const int b = blockIdx.x;
  return H % 8 == 0 ? (b % 8) * (H / 8) + b / 8 : b;
}

// The first wave works out a chunk's steps and sums of logarithms: dt [64] (0 behind the chunk's end), the sums as two
// floats each.
__device__ __forceinline__ void ss_steps(const float* __restrict__ dt_pre, long dt_stride, int h, int nt, float bias,
                                         float rate, float* sdt, float* shi, float* slo) {
  if (threadIdx.x >= SS_L) return;
  const int t = threadIdx.x;
  const float dt = t < nt ? ss_softplus(dt_pre[(long)t * dt_stride + h] + bias) : 0.f;
  double c = -(double)rate * (double)dt;
#pragma unroll
  for (int o = 1; o < SS_L; o <<= 1) {
    const double up = __shfl_up(c, o, LMSF_WAVE);
    if (t >= o) c += up;
  }
  const float hi = (float)c;
  sdt[t] = dt;
  shi[t] = hi;
  slo[t] = (float)(c - (double)hi);
}

// Entry i of the chunks' list: chunks[3 i .. 3 i + 2] = first token, number of tokens, segment.
// U of a chunk and head, in [dv][N], and exp(c_L). Four waves; a wave takes 16 value entries at a time against all N.
__global__ __launch_bounds__(256) void state_space_sums_kernel(
    const bf16_t* __restrict__ xbc, long xbc_stride, int x_at, int b_at, const float* __restrict__ dt_pre, long dt_stride,
    const float* __restrict__ dt_bias, const float* __restrict__ rate, const int* __restrict__ chunks,
    float* __restrict__ U, float* __restrict__ decay, int H, int G, int N, int dv, int vec_b, int vec_x) {
  extern __shared__ __align__(16) unsigned char lds[];
  const int Np = (N + 15) / 16 * 16, dvp = (dv + 15) / 16 * 16;
  unsigned char* BT = lds;                        // [Np][64] turned
  unsigned char* XT = BT + Np * 128;              // [dvp][64] turned
  float* sdt = reinterpret_cast<float*>(XT + dvp * 128);
  float* shi = sdt + SS_L;
  float* slo = shi + SS_L;
  float* sw = slo + SS_L;                         // [64]: exp(c_L - c_u) dt_u
  const int h = ss_head(H), g = h / (H / G);
  const long i = blockIdx.y;
  const int t0 = chunks[3 * i], nt = chunks[3 * i + 1];
  ss_stage_turned(xbc + (long)t0 * xbc_stride + b_at + g * N, xbc_stride, nt, N, Np, vec_b, BT);
  ss_stage_turned(xbc + (long)t0 * xbc_stride + x_at + h * dv, xbc_stride, nt, dv, dvp, vec_x, XT);
  ss_steps(dt_pre + (long)t0 * dt_stride, dt_stride, h, nt, dt_bias[h], rate[h], sdt, shi, slo);
  __syncthreads();
  if (threadIdx.x < SS_L) {
    const int u = threadIdx.x;
    // (tokens behind the chunk's end have dt = 0: the last sum is the chunk's, and their weight is 0)
    sw[u] = sdt[u] * expf((shi[SS_L - 1] - shi[u]) + (slo[SS_L - 1] - slo[u]));
    if (u == 0) decay[i * H + h] = expf(shi[SS_L - 1] + slo[SS_L - 1]);
  }
  __syncthreads();
  const int wave = threadIdx.x / LMSF_WAVE, lane = threadIdx.x % LMSF_WAVE, fr = lane % 16, fg = lane / 16;
  float* out = U + (i * H + h) * (long)dv * N;
  for (int et = wave; et < dvp / 16; et += 4) {
    SsFrag xa[2][3];
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      SsFrag raw;
      raw.q = *reinterpret_cast<const uint4*>(XT + ss_turned(et * 16 + fr, k * 4 + fg));
      float v[8];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        v[2 * j] = __uint_as_float(raw.w[j] << 16) * sw[k * 32 + fg * 8 + 2 * j];
        v[2 * j + 1] = __uint_as_float(raw.w[j] & 0xffff0000u) * sw[k * 32 + fg * 8 + 2 * j + 1];
      }
      ss_parts8(v, xa[k]);
    }
    for (int nb = 0; nb < Np / 16; ++nb) {
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        SsFrag b;
        b.q = *reinterpret_cast<const uint4*>(BT + ss_turned(nb * 16 + fr, k * 4 + fg));
#pragma unroll
        for (int p = 0; p < 3; ++p) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xa[k][p].v, b.v, acc, 0, 0, 0);
      }
      const int n = nb * 16 + fr;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int e = et * 16 + fg * 4 + r;
        if (n < N && e < dv) out[(long)e * N + n] = acc[r];
      }
    }
  }
}

// Chunk after chunk of a segment: S_0 takes U's place, S <- exp(c_L) S + U; at the end S goes to the slot. A thread V
// neighbours of one head's state. bases[s], bases[s + 1]: a segment's entries.
template <int V>
__global__ __launch_bounds__(256) void state_space_fold_kernel(float* __restrict__ state, long state_stride,
                                                               const int* __restrict__ state_slots,
                                                               const int* __restrict__ bases, float* __restrict__ U,
                                                               const float* __restrict__ decay, int H, long per) {
  const int h = blockIdx.y, s = blockIdx.z;
  const long i = ((long)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= per) return;
  float* st = state + (long)state_slots[s] * state_stride + (long)h * per + i;
  float S[V];
#pragma unroll
  for (int j = 0; j < V; ++j) S[j] = st[j];
  const int c1 = bases[s + 1];
  constexpr int AHEAD = 4;
  for (int c = bases[s]; c < c1; c += AHEAD) {
    float u[AHEAD][V], dk[AHEAD];
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      const long ent = (long)min(c + a, c1 - 1) * H + h;
      dk[a] = decay[ent];
#pragma unroll
      for (int j = 0; j < V; ++j) u[a][j] = U[ent * per + i + j];
    }
#pragma unroll
    for (int a = 0; a < AHEAD; ++a) {
      if (c + a >= c1) break;
      float* p = U + ((long)(c + a) * H + h) * per + i;
#pragma unroll
      for (int j = 0; j < V; ++j) {
        p[j] = S[j];
        S[j] = fmaf(dk[a], S[j], u[a][j]);
      }
    }
  }
#pragma unroll
  for (int j = 0; j < V; ++j) st[j] = S[j];
}

// The outputs of a chunk and head. First every wave makes the decayed and stepped C . B of its 16 tokens (C . B turned:
// rows u, columns t) and leaves its three bfloat16 parts in LDS as the second product takes them; then a wave takes 16
// value entries at a time against all 64 tokens.
// PT: [4 blocks of 16 t][2 pairs of u blocks][3 parts][64 lanes] of 16 bytes.
__global__ __launch_bounds__(256, 3) void state_space_outputs_kernel(
    const bf16_t* __restrict__ xbc, long xbc_stride, int x_at, int b_at, int c_at, const float* __restrict__ dt_pre,
    long dt_stride, const float* __restrict__ dt_bias, const float* __restrict__ rate, const float* __restrict__ D,
    const int* __restrict__ chunks, const float* __restrict__ S0, float* __restrict__ y, long y_stride, int H, int G, int N,
    int dv, int vec_b, int vec_x, int vec_s, int vec_y) {
  extern __shared__ __align__(16) unsigned char lds[];
  const int Nk = (N + 31) / 32 * 32, dvp = (dv + 15) / 16 * 16, row_bytes = Nk * 2 + 16;
  unsigned char* Cs = lds;                              // [64][row_bytes]
  unsigned char* Bs = Cs + SS_L * row_bytes;            // [64][row_bytes]
  unsigned char* XT = Bs + max(SS_L * row_bytes, SS_PT);   // [dvp][64] turned
  unsigned char* PT = Bs;                               // (takes B's place once every wave has multiplied)
  float* sdt = reinterpret_cast<float*>(XT + dvp * 128);
  float* shi = sdt + SS_L;
  float* slo = shi + SS_L;
  const int h = ss_head(H), g = h / (H / G);
  const long i = blockIdx.y;
  const int t0 = chunks[3 * i], nt = chunks[3 * i + 1];
  const int wave = threadIdx.x / LMSF_WAVE, lane = threadIdx.x % LMSF_WAVE, fr = lane % 16, fg = lane / 16;
  const float* S = S0 + (i * H + h) * (long)dv * N;
  const int nk = Nk / 32;
  // the state's numbers of the wave's first 16 value entries are asked for first
  auto load_state = [&](int et, int k, float* v) {
    const int e = et * 16 + fr, n = k * 32 + fg * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = 0.f;
    if (e >= dv) return;
    const float* p = S + (long)e * N + n;
    if (vec_s) {
      if (n < N) ss_load4(p, v), ss_load4(p + 4, v + 4);
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (n + j < N) v[j] = p[j];
    }
  };
  float ahead[4][8];
#pragma unroll
  for (int k = 0; k < 4; ++k)
    if (k < nk) load_state(wave, k, ahead[k]);
  const bf16_t* base = xbc + (long)t0 * xbc_stride;
  ss_stage_two(base + c_at + g * N, base + b_at + g * N, xbc_stride, nt, N, Nk, vec_b, Cs, SS_L * row_bytes, row_bytes);
  ss_stage_turned(base + x_at + h * dv, xbc_stride, nt, dv, dvp, vec_x, XT);
  ss_steps(dt_pre + (long)t0 * dt_stride, dt_stride, h, nt, dt_bias[h], rate[h], sdt, shi, slo);
  __syncthreads();
  {
    const int t = wave * 16 + fr;                        // this lane's token
    f32x4_t p[4];
#pragma unroll
    for (int ub = 0; ub < 4; ++ub) p[ub] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < nk; ++k) {
      SsFrag cf;
      cf.q = *reinterpret_cast<const uint4*>(Cs + t * row_bytes + k * 64 + fg * 16);
#pragma unroll
      for (int ub = 0; ub < 4; ++ub) {
        if (ub > wave) continue;
        SsFrag bf;
        bf.q = *reinterpret_cast<const uint4*>(Bs + (ub * 16 + fr) * row_bytes + k * 64 + fg * 16);
        p[ub] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf.v, cf.v, p[ub], 0, 0, 0);
      }
    }
    const float hi = shi[t], lo = slo[t];
    __syncthreads();
#pragma unroll
    for (int pair = 0; pair < 2; ++pair) {
      if (pair * 2 > wave) continue;
      float v[8];
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int u = (pair * 2 + b) * 16 + fg * 4 + r;
          v[b * 4 + r] = u <= t ? p[pair * 2 + b][r] * (sdt[u] * expf((hi - shi[u]) + (lo - slo[u]))) : 0.f;
        }
      SsFrag f[3];
      ss_parts8(v, f);
#pragma unroll
      for (int q = 0; q < 3; ++q)
        *reinterpret_cast<uint4*>(PT + ((((wave * 2 + pair) * 3 + q) * 64 + lane) << 4)) = f[q].q;
    }
  }
  __syncthreads();
  const float skip = D[h];
  for (int et = wave; et < dvp / 16; et += 4) {
    f32x4_t acc[4];
#pragma unroll
    for (int tb = 0; tb < 4; ++tb) acc[tb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    auto with_state = [&](int k, const float* v) {
      SsFrag f[3];
      ss_parts8(v, f);
#pragma unroll
      for (int tb = 0; tb < 4; ++tb) {
        SsFrag cf;
        cf.q = *reinterpret_cast<const uint4*>(Cs + (tb * 16 + fr) * row_bytes + k * 64 + fg * 16);
#pragma unroll
        for (int q = 0; q < 3; ++q) acc[tb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f[q].v, cf.v, acc[tb], 0, 0, 0);
      }
      __builtin_amdgcn_sched_barrier(0);      // (else the scheduler asks for all blocks' operands at once and runs out of registers)
    };
    if (et != wave) {
#pragma unroll
      for (int k = 0; k < 4; ++k)
        if (k < nk) load_state(et, k, ahead[k]);
    }
#pragma unroll
    for (int k = 0; k < 4; ++k)
      if (k < nk) with_state(k, ahead[k]);
    for (int k = 4; k < nk; ++k) {
      float v[8];
      load_state(et, k, v);
      with_state(k, v);
    }
#pragma unroll
    for (int tb = 0; tb < 4; ++tb) {
      const int t = tb * 16 + fr;
      acc[tb] *= expf(shi[t] + slo[t]);
#pragma unroll
      for (int pair = 0; pair < 2; ++pair) {
        if (pair * 2 > tb) continue;
        // x turned: row e, the tokens 4 fg .. + 3 of both blocks of the pair
        const int c = et * 16 + fr, u0 = pair * 32 + fg * 4, u1 = u0 + 16;
        SsFrag xf;
        xf.h[0] = *reinterpret_cast<const uint2*>(XT + ss_turned(c, u0 >> 3) + (u0 & 7) * 2);
        xf.h[1] = *reinterpret_cast<const uint2*>(XT + ss_turned(c, u1 >> 3) + (u1 & 7) * 2);
#pragma unroll
        for (int q = 0; q < 3; ++q) {
          SsFrag pf;
          pf.q = *reinterpret_cast<const uint4*>(PT + ((((tb * 2 + pair) * 3 + q) * 64 + lane) << 4));
          acc[tb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xf.v, pf.v, acc[tb], 0, 0, 0);
        }
      }
      if (t < nt) {
        // this lane: token t, value entries 4 fg .. + 3
        float o[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int c = et * 16 + fg * 4 + r;
          const bf16_t xv = *reinterpret_cast<const bf16_t*>(XT + ss_turned(c, t >> 3) + (t & 7) * 2);
          o[r] = fmaf(skip, bf16_to_f32(xv), acc[tb][r]);
        }
        float* out = y + (long)(t0 + t) * y_stride + (long)h * dv + et * 16 + fg * 4;
        if (vec_y) {
          if (et * 16 + fg * 4 < dv) *reinterpret_cast<float4*>(out) = make_float4(o[0], o[1], o[2], o[3]);
        } else {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            if (et * 16 + fg * 4 + r < dv) out[r] = o[r];
        }
      }
      __builtin_amdgcn_sched_barrier(0);
    }
  }
}

static size_t ss_sums_smem(int N, int dv) {
  return (size_t)((N + 15) / 16 * 16 + (dv + 15) / 16 * 16) * 128 + 4 * SS_L * sizeof(float);
}
static size_t ss_outputs_smem(int N, int dv) {
  const int rows = SS_L * ((N + 31) / 32 * 64 + 16);
  return (size_t)rows + (rows > SS_PT ? rows : SS_PT) + (size_t)(dv + 15) / 16 * 16 * 128 + 3 * SS_L * sizeof(float);
}

// tokens of a chunk of the chunked form; 0: its operands do not fit a workgroup's LDS (or the run is float32)
extern "C" int lmsf_state_space_chunk_tokens(int dtype, int N, int dv) {
  return dtype == LMSF_BF16 && ss_sums_smem(N, dv) <= 150 * 1024 && ss_outputs_smem(N, dv) <= 150 * 1024 ? SS_L : 0;
}

// floats of scratch a chunk takes: U, and a decay a head
extern "C" long lmsf_state_space_entry_floats(int H, int N, int dv) { return (long)H * N * dv + H; }

static int ss_check(const void* xbc, int dtype, long xbc_stride, int x_at, int b_at, int c_at, const float* dt_pre,
                    long dt_stride, const float* dt_bias, const float* rate, const float* D, float* state,
                    long state_stride, const int* state_slots, float* y, long y_stride, int n_tokens, int n_segments, int H,
                    int G, int N, int dv) {
  LMSF_CHECK(xbc && dt_pre && dt_bias && rate && D && state && state_slots && y, "state_space: null pointer");
  LMSF_CHECK(dtype == LMSF_F32 || dtype == LMSF_BF16, "state_space: unknown dtype code %d", dtype);
  LMSF_CHECK(H > 0 && H <= 65535 && G > 0 && H % G == 0 && N > 0 && N <= SS_MAX_STATE && dv > 0 && dv <= 65535,
             "state_space: bad sizes H=%d G=%d N=%d dv=%d", H, G, N, dv);
  LMSF_CHECK(x_at >= 0 && b_at >= 0 && c_at >= 0 && xbc_stride >= (long)x_at + (long)H * dv &&
                 xbc_stride >= (long)b_at + (long)G * N && xbc_stride >= (long)c_at + (long)G * N && dt_stride >= H &&
                 y_stride >= (long)H * dv && state_stride >= lmsf_state_space_state_floats(H, N, dv),
             "state_space: strides too small");
  LMSF_CHECK(n_tokens >= 0 && n_segments >= 0 && n_segments <= 65535, "state_space: bad counts");
  return 0;
}

// xbc [n_tokens, >= ...] of ``dtype``: x in columns x_at .. (heads of dv), B in b_at .. and C in c_at .. (G groups of N);
// dt_pre float32 [n_tokens, >= H]; dt_bias, rate, D float32 [H]; y float32 [n_tokens, H * dv]. Segment s holds the tokens
// seg_starts[s] .. seg_starts[s + 1] - 1 and the state of slot state_slots[s].
extern "C" int lmsf_state_space_tokens(const void* xbc, int dtype, long xbc_stride, int x_at, int b_at, int c_at,
                                       const float* dt_pre, long dt_stride, const float* dt_bias, const float* rate,
                                       const float* D, float* state, long state_stride, const int* seg_starts,
                                       const int* state_slots, float* y, long y_stride, int n_tokens, int n_segments, int H,
                                       int G, int N, int dv, hipStream_t stream) {
  if (ss_check(xbc, dtype, xbc_stride, x_at, b_at, c_at, dt_pre, dt_stride, dt_bias, rate, D, state, state_stride,
               state_slots, y, y_stride, n_tokens, n_segments, H, G, N, dv))
    return 1;
  LMSF_CHECK(seg_starts, "state_space: null pointer");
  if (n_tokens == 0 || n_segments == 0) return 0;
  const int al = dtype == LMSF_F32 ? 16 : 8;      // bytes of four entries
  const bool vec = N % 4 == 0 && state_stride % 4 == 0 && lmsf_aligned16(state) && xbc_stride % 4 == 0 && b_at % 4 == 0 &&
                   c_at % 4 == 0 && ((uintptr_t)xbc) % al == 0;
  const int quads = (N + 3) / 4;
#define SS_TOK(T, LPR, K, R, V)                                                                                        \
  hipLaunchKernelGGL((state_space_token_kernel<T, LPR, K, R, V>),                                                      \
                     dim3((dv + 256 / LPR * R - 1) / (256 / LPR * R), H, n_segments), dim3(256), 0, stream,            \
                     (const T*)xbc, xbc_stride, x_at, b_at, c_at, dt_pre, dt_stride, dt_bias, rate, D, state,          \
                     state_stride, seg_starts, state_slots, y, y_stride, H, G, N, dv)
  // few heads and requests: two value entries a group of lanes, so that more workgroups share the state
#define SS_TOK_R(T, LPR, K)                                                                                            \
  do {                                                                                                                 \
    const bool small = (long)H * n_segments * ((dv + 256 / LPR * 4 - 1) / (256 / LPR * 4)) < 1024;                     \
    if (small) { if (vec) SS_TOK(T, LPR, K, 2, true); else SS_TOK(T, LPR, K, 2, false); }                              \
    else { if (vec) SS_TOK(T, LPR, K, 4, true); else SS_TOK(T, LPR, K, 4, false); }                                    \
  } while (0)
#define SS_TOK_T(T)                                \
  do {                                             \
    if (quads <= 4) SS_TOK_R(T, 4, 1);             \
    else if (quads <= 8) SS_TOK_R(T, 8, 1);        \
    else if (quads <= 16) SS_TOK_R(T, 16, 1);      \
    else if (quads <= 32) SS_TOK_R(T, 32, 1);      \
    else if (quads <= 64) SS_TOK_R(T, 64, 1);      \
    else if (quads <= 128) SS_TOK_R(T, 64, 2);     \
    else SS_TOK_R(T, 64, 4);                       \
  } while (0)
  if (dtype == LMSF_F32) SS_TOK_T(float); else SS_TOK_T(bf16_t);
#undef SS_TOK_T
#undef SS_TOK_R
#undef SS_TOK
  LMSF_LAUNCH_CHECK("state_space_tokens");
  return 0;
}

// The same function in chunks (bfloat16). ``chunks`` int32 [n_chunks, 3] = first token, number of tokens (at most
// lmsf_state_space_chunk_tokens), segment: a segment's chunks in order, the segments in order; ``bases`` int32
// [n_segments + 1]: a segment's first chunk; ``entries``: n_chunks * lmsf_state_space_entry_floats floats.
extern "C" int lmsf_state_space_chunked(const void* xbc, int dtype, long xbc_stride, int x_at, int b_at, int c_at,
                                        const float* dt_pre, long dt_stride, const float* dt_bias, const float* rate,
                                        const float* D, float* state, long state_stride, const int* state_slots,
                                        const int* chunks, const int* bases, int n_chunks, float* entries, float* y,
                                        long y_stride, int n_tokens, int n_segments, int H, int G, int N, int dv,
                                        hipStream_t stream) {
  if (ss_check(xbc, dtype, xbc_stride, x_at, b_at, c_at, dt_pre, dt_stride, dt_bias, rate, D, state, state_stride,
               state_slots, y, y_stride, n_tokens, n_segments, H, G, N, dv))
    return 1;
  LMSF_CHECK(lmsf_state_space_chunk_tokens(dtype, N, dv) > 0, "state_space: states of %d x %d have no chunked form", N, dv);
  LMSF_CHECK(chunks && bases && entries && n_chunks >= n_segments && n_chunks <= 65535, "state_space: bad list of chunks");
  if (n_tokens == 0 || n_segments == 0) return 0;
  const long per = (long)N * dv;
  float* decay = entries + (long)n_chunks * H * per;
  const bool rows8 = xbc_stride % 8 == 0 && lmsf_aligned16(xbc);
  const int vec_b = rows8 && N % 8 == 0 && b_at % 8 == 0 && c_at % 8 == 0;
  const int vec_x = rows8 && dv % 8 == 0 && x_at % 8 == 0;
  const int vec_s = N % 8 == 0 && lmsf_aligned16(entries);
  const int vec_y = dv % 4 == 0 && y_stride % 4 == 0 && lmsf_aligned16(y);
  const size_t smem1 = ss_sums_smem(N, dv), smem2 = ss_outputs_smem(N, dv);
  static size_t reserved1 = 0, reserved2 = 0;
  hipError_t e = hipSuccess;
  if (smem1 > 64 * 1024 && smem1 > reserved1) {
    e = hipFuncSetAttribute(reinterpret_cast<const void*>(state_space_sums_kernel),
                            hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem1);
    reserved1 = smem1;
  }
  if (e == hipSuccess && smem2 > 64 * 1024 && smem2 > reserved2) {
    e = hipFuncSetAttribute(reinterpret_cast<const void*>(state_space_outputs_kernel),
                            hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem2);
    reserved2 = smem2;
  }
  if (e != hipSuccess) {
    reserved1 = reserved2 = 0;
    lmsf_set_error("state_space: cannot reserve LDS: %s", hipGetErrorString(e));
    return 2;
  }
  hipLaunchKernelGGL(state_space_sums_kernel, dim3(H, n_chunks), dim3(256), smem1, stream, (const bf16_t*)xbc, xbc_stride,
                     x_at, b_at, dt_pre, dt_stride, dt_bias, rate, chunks, entries, decay, H, G, N, dv, vec_b, vec_x);
  LMSF_LAUNCH_CHECK("state_space_sums");
  if (per % 4 == 0 && state_stride % 4 == 0 && lmsf_aligned16(state) && lmsf_aligned16(entries))
    hipLaunchKernelGGL((state_space_fold_kernel<4>), dim3((unsigned)((per / 4 + 255) / 256), H, n_segments), dim3(256), 0,
                       stream, state, state_stride, state_slots, bases, entries, decay, H, per);
  else
    hipLaunchKernelGGL((state_space_fold_kernel<1>), dim3((unsigned)((per + 255) / 256), H, n_segments), dim3(256), 0,
                       stream, state, state_stride, state_slots, bases, entries, decay, H, per);
  LMSF_LAUNCH_CHECK("state_space_fold");
  hipLaunchKernelGGL(state_space_outputs_kernel, dim3(H, n_chunks), dim3(256), smem2, stream, (const bf16_t*)xbc,
                     xbc_stride, x_at, b_at, c_at, dt_pre, dt_stride, dt_bias, rate, D, chunks, entries, y, y_stride, H, G,
                     N, dv, vec_b, vec_x, vec_s, vec_y);
  LMSF_LAUNCH_CHECK("state_space_outputs");
  return 0;
}

// ---------------------------------------------------------------- the gate and the norm behind it
// out[n] = gn(y[n] silu(z[n]); w): the row is gated, then cut into ``parts`` equal pieces, each over its own root mean
// square (eps inside the root), times w [inner]. A workgroup a row and piece.
template <typename T>
__global__ __launch_bounds__(1024) void gated_group_norm_kernel(const float* __restrict__ y, long y_stride,
                                                                const T* __restrict__ z, long z_stride,
                                                                const float* __restrict__ w, T* __restrict__ out,
                                                                long out_stride, int part, float eps, int vec) {
  extern __shared__ float row[];      // [part]
  __shared__ float red[16];
  const long n = blockIdx.x;
  const int at = blockIdx.y * part, threads = blockDim.x;
  float ss = 0.f;
  if (vec) {
    for (int i = threadIdx.x * 4; i < part; i += threads * 4) {
      float a[4], g[4];
      ss_load4(y + n * y_stride + at + i, a);
      ss_load4(z + n * z_stride + at + i, g);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        a[j] *= g[j] / (1.f + expf(-g[j]));
        ss = fmaf(a[j], a[j], ss);
        row[i + j] = a[j];
      }
    }
  } else {
    for (int i = threadIdx.x; i < part; i += threads) {
      const float g = to_f32<T>(z[n * z_stride + at + i]);
      const float a = y[n * y_stride + at + i] * (g / (1.f + expf(-g)));
      ss = fmaf(a, a, ss);
      row[i] = a;
    }
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)part + eps);
  // (each thread reads back what it wrote itself)
  if (vec) {
    for (int i = threadIdx.x * 4; i < part; i += threads * 4) {
      float wv[4];
      ss_load4(w + at + i, wv);
#pragma unroll
      for (int j = 0; j < 4; ++j) wv[j] *= row[i + j] * inv;
      ss_store4(out + n * out_stride + at + i, wv);
    }
  } else {
    for (int i = threadIdx.x; i < part; i += threads) out[n * out_stride + at + i] = from_f32<T>(w[at + i] * (row[i] * inv));
  }
}

extern "C" int lmsf_gated_group_norm(const float* y, long y_stride, const void* z, long z_stride, int dtype, const float* w,
                                     void* out, long out_stride, int n_rows, int inner, int parts, float eps,
                                     hipStream_t stream) {
  LMSF_CHECK(y && z && w && out, "gated_group_norm: null pointer");
  LMSF_CHECK(dtype == LMSF_F32 || dtype == LMSF_BF16, "gated_group_norm: unknown dtype code %d", dtype);
  LMSF_CHECK(inner > 0 && parts > 0 && parts <= 65535 && inner % parts == 0, "gated_group_norm: %d columns do not split into %d parts",
             inner, parts);
  const int part = inner / parts;
  LMSF_CHECK(part <= 16384 - 16, "gated_group_norm: parts of %d columns (at most 16,368)", part);
  LMSF_CHECK(y_stride >= inner && z_stride >= inner && out_stride >= inner, "gated_group_norm: rows overlap");
  if (n_rows <= 0) return 0;
  const int es = lmsf_elem_size(dtype);
  const int vec = part % 4 == 0 && y_stride % 4 == 0 && z_stride % 4 == 0 && out_stride % 4 == 0 && lmsf_aligned16(y) &&
                  lmsf_aligned16(w) && ((uintptr_t)z) % (4 * es) == 0 && ((uintptr_t)out) % (4 * es) == 0;
  int threads = 64;
  const int most = n_rows * parts >= 1024 ? 256 : 1024;
  while (threads < most && threads * 4 < part) threads *= 2;
  const dim3 grid(n_rows, parts);
  if (dtype == LMSF_F32)
    hipLaunchKernelGGL((gated_group_norm_kernel<float>), grid, dim3(threads), (size_t)part * 4, stream, y, y_stride,
                       (const float*)z, z_stride, w, (float*)out, out_stride, part, eps, vec);
  else
    hipLaunchKernelGGL((gated_group_norm_kernel<bf16_t>), grid, dim3(threads), (size_t)part * 4, stream, y, y_stride,
                       (const bf16_t*)z, z_stride, w, (bf16_t*)out, out_stride, part, eps, vec);
  LMSF_LAUNCH_CHECK("gated_group_norm");
  return 0;
}
