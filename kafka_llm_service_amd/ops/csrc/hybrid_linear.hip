// Kernels of linear-attention recurrences with per-channel decays and of post-normed residuals, for gfx950.
//
// Every kernel is built for bf16 and for fp32 activations; decays and their logarithms, step sizes, unit norms, norm
// statistics, the recurrent state and every product it takes part in are fp32 in both. Sizes are run-time values with
// no alignment assumptions. A step's rows are described by segments (seg[r] = first row, rows, first position, state
// slot); a segment whose first position is 0 starts from a zero state: its slot is written, never read.
//
//   norm_add     x += rms_norm(y1 + y2) * w on the fp32 stream, the new x also in the activation dtype; y1 may be the
//                split-K slabs of a projection (summed while loading)
//   relu2        the square of relu;  silu_mul   silu(gate) * up
//   The recurrence S_t = diag(a_t) S_(t-1) + k_t u_t^T, o_t = S_t^T q_t per head, in two forms:
//     gated linear attention   u = v, a = sigmoid(z)^(1 / tau)
//     gated delta rule         u = beta (v - (diag(a_t) S_(t-1))^T k_t), a = exp(rate_h softplus(z)), q and k unit vectors
//   lin_scan     token by token: one workgroup per (segment, head, 64 value columns), a wave owns 16 columns (a thread:
//                a quarter of the rows of one column, in registers), so that the row sums stay inside the wave; 8
//                tokens' inputs are staged in LDS, double buffered, one barrier per block
//   lin_step     segments of one token (decode): the state moves through registers once in 16-byte pieces
//   lin_chunk_prep / lin_chunk_scan   long segments in chunks of 32 tokens. With b_t the running sum of the chunk's log
//                decays, the chunk's outputs and its new state are matrix products:
//                  P[t][j] = q_t . (k_j e^(b_t - b_j)) (j <= t),  A[t][j] = beta_t k_t . (k_j e^(b_t - b_j)) (j < t)
//                  U = V,  or for the delta rule  (I + A) U = diag(beta) (V - (K e^b) S), i.e. U = U0 - W S with
//                  [W | U0] = (I + A)^(-1) diag(beta) [K e^b | V]
//                  O = (Q e^b) S + P U,   S <- diag(e^(b_end)) S + (K e^(b_end - b))^T U
//                prep computes everything that does not depend on S for all chunks in parallel; scan walks a
//                sequence's chunks with 16 value columns of S in the accumulators of a workgroup, all products on
//                the fp32 matrix cores.
#include "common.h"

namespace kafka {
namespace hl {

template <typename T>
__device__ __forceinline__ float ldf(const T* p) { return (float)(*p); }
template <typename T>
__device__ __forceinline__ void stf(T* p, float v) { *p = (T)v; }

constexpr int NT = 256;
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplusf(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// Workgroup barrier for LDS hand-overs that leaves global loads (a prefetched next block) in flight: __syncthreads()
// would drain them as well. This wave's LDS reads and writes are complete (lgkmcnt 0) before it arrives.
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// ---- post-normed residual -------------------------------------------------------------------------------------------
constexpr int NA_MAXS = 8;   // split-K slabs of y1

// One workgroup per row. VEC consecutive columns per thread and round, NV rounds in registers (d <= NT VEC NV): every
// load of the row is in flight before the statistics, the sublayer's output and the residual stay in registers. S: slabs of
// an fp32 y1, 0 = y1 in the activation dtype.
template <typename AT, int VEC, int NV, int S>
__global__ __launch_bounds__(NT) void norm_add_kernel(float* __restrict__ x, int64_t xs, const void* __restrict__ y1,
                                                      int64_t y1s, int64_t slab,
                                                      const AT* __restrict__ y2, int64_t y2s,
                                                      const float* __restrict__ w, float eps, AT* __restrict__ out,
                                                      int64_t os, int d) {
  __shared__ float red[NT / 64];
  const int64_t t = blockIdx.x;
  float* xr = x + t * xs;
  float yv[NV][VEC], xv[NV][VEC];
  float acc = 0.f;
#pragma unroll
  for (int it = 0; it < NV; ++it) {
    const int i = (it * NT + threadIdx.x) * VEC;
#pragma unroll
    for (int e = 0; e < VEC; ++e) yv[it][e] = xv[it][e] = 0.f;
    if (i < d) {
      if constexpr (S > 0) {
        const float* p = reinterpret_cast<const float*>(y1) + t * y1s + i;
#pragma unroll
        for (int s = 0; s < S; ++s) {
#pragma unroll
          for (int e = 0; e < VEC; ++e) yv[it][e] += p[s * slab + e];
        }
      } else {
        const AT* p = reinterpret_cast<const AT*>(y1) + t * y1s + i;
#pragma unroll
        for (int e = 0; e < VEC; ++e) yv[it][e] = ldf(p + e);
      }
      if (y2 != nullptr) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) yv[it][e] += ldf(y2 + t * y2s + i + e);
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) xv[it][e] = xr[i + e];
    }
  }
#pragma unroll
  for (int it = 0; it < NV; ++it)
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc += yv[it][e] * yv[it][e];
  const float rs = 1.0f / sqrtf(block_sum<NT>(acc, red) / (float)d + eps);
#pragma unroll
  for (int it = 0; it < NV; ++it) {
    const int i = (it * NT + threadIdx.x) * VEC;
    if (i < d) {
      float v[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] = xv[it][e] + yv[it][e] * rs * w[i + e];
#pragma unroll
      for (int e = 0; e < VEC; ++e) xr[i + e] = v[e];
      if (out != nullptr) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) stf(out + t * os + i + e, v[e]);
      }
    }
  }
}

// rows of any width: two passes over the sublayer's output
template <typename AT>
__global__ __launch_bounds__(NT) void norm_add_wide_kernel(float* __restrict__ x, int64_t xs,
                                                           const void* __restrict__ y1, int64_t y1s, int y1_f32, int S,
                                                           int64_t slab, const AT* __restrict__ y2, int64_t y2s,
                                                           const float* __restrict__ w, float eps,
                                                           AT* __restrict__ out, int64_t os, int d) {
  __shared__ float red[NT / 64];
  const int64_t t = blockIdx.x;
  auto y = [&](int i) {
    float v = 0.f;
    if (y1_f32) {
      for (int s = 0; s < S; ++s) v += reinterpret_cast<const float*>(y1)[s * slab + t * y1s + i];
    } else {
      v = ldf(reinterpret_cast<const AT*>(y1) + t * y1s + i);
    }
    return y2 != nullptr ? v + ldf(y2 + t * y2s + i) : v;
  };
  float acc = 0.f;
  for (int i = threadIdx.x; i < d; i += NT) {
    const float v = y(i);
    acc += v * v;
  }
  const float rs = 1.0f / sqrtf(block_sum<NT>(acc, red) / (float)d + eps);
  for (int i = threadIdx.x; i < d; i += NT) {
    const float v = x[t * xs + i] + y(i) * rs * w[i];
    x[t * xs + i] = v;
    if (out != nullptr) stf(out + t * os + i, v);
  }
}

// ---- element-wise feed-forward activations ------------------------------------------------------------------------
template <typename AT>
__global__ void relu2_kernel(const AT* __restrict__ u, int64_t us, AT* __restrict__ out, int64_t os, int64_t T, int F) {
  const int64_t n = T * F;
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t t = i / F;
    const int f = (int)(i - t * F);
    const float v = fmaxf(ldf(u + t * us + f), 0.f);
    stf(out + t * os + f, v * v);
  }
}

template <typename AT>
__global__ void silu_mul_kernel(const AT* __restrict__ gu, int64_t gs, AT* __restrict__ out, int64_t os, int64_t T,
                                int F) {
  const int64_t n = T * F;
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t t = i / F;
    const int f = (int)(i - t * F);
    const float g = ldf(gu + t * gs + f);
    stf(out + t * os + f, g / (1.0f + expf(-g)) * ldf(gu + t * gs + F + f));
  }
}

// the same on bf16 rows whose sizes, strides and bases are multiples of 8 elements (GLU: silu(gate) * up, else relu^2)
template <bool GLU>
__global__ void act_vec8_kernel(const bf16* __restrict__ u, int64_t us, bf16* __restrict__ out, int64_t os, int64_t T,
                                int F) {
  const int F8 = F >> 3;
  const int64_t n = T * F8;
  for (int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (int64_t)gridDim.x * blockDim.x) {
    const int64_t t = i / F8;
    const int f = (int)(i - t * F8) << 3;
    const bf16x8 a = load_bf16x8(u + t * us + f);
    bf16x8 o;
    if constexpr (GLU) {
      const bf16x8 b = load_bf16x8(u + t * us + F + f);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float g = (float)a[j];
        o[j] = (bf16)(g / (1.0f + expf(-g)) * (float)b[j]);
      }
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float v = fmaxf((float)a[j], 0.f);
        o[j] = (bf16)(v * v);
      }
    }
    store_bf16x8(out + t * os + f, o);
  }
}

// ---- the recurrence's inputs ------------------------------------------------------------------------------------------
// Row t: query / key head g at qk + t qk_s + q_off (k_off) + g D; value head h at v + t v_s + h Dv; raw decay at z + t
// z_s + h D (+ z_bias); raw beta at beta + t beta_s + h. Head h uses query / key head h / (H / G).
template <typename AT>
struct LinIn {
  const AT* qk;
  const AT* v;
  const AT* z;
  const AT* beta;
  const float* z_bias;   // [H D]
  const float* rate;     // [H], delta rule: log a = rate softplus(z + bias)
  int64_t qk_s, v_s, z_s, beta_s;
  int q_off, k_off, H, G, D, Dv;
  float qscale, inv_tau;
};

template <bool DELTA>
__device__ __forceinline__ float log_decay(float z, float rate, float inv_tau) {
  return DELTA ? rate * softplusf(z) : -softplusf(-z) * inv_tau;
}
constexpr float UNIT_EPS = 1e-6f;

// ---- token by token --------------------------------------------------------------------------------------------------
constexpr int LS_TB = 8;   // tokens per staged block

template <typename AT, int RD, bool DELTA>
__global__ __launch_bounds__(NT) void lin_scan_kernel(LinIn<AT> in, const int* __restrict__ seg, int min_n,
                                                      int max_n, float* __restrict__ Sst, float* __restrict__ out, int64_t os) {
  constexpr int DMAX = 4 * RD;
  constexpr int LROW = DMAX + 16;            // a row group's rows are shifted by 4 floats: reads of the groups spread
  constexpr int NE = (DMAX + 63) / 64;       // elements of a staged row per lane
  __shared__ __attribute__((aligned(16))) float st[2][LS_TB][3][LROW];   // q, k, decay
  __shared__ float vs[2][LS_TB][64];
  __shared__ float bs[2][LS_TB];
  const int r = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * 64;
  const int q0 = seg[4 * r], n = seg[4 * r + 1], p0 = seg[4 * r + 2], slot = seg[4 * r + 3];
  if (n > max_n || n < min_n) return;   // (uniform) a segment that the chunk or the step kernel takes
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, rg = lane >> 4;
  const int col = w * 16 + (lane & 15);
  const bool vok = v0 + col < in.Dv;
  const int D = in.D, g = h / (in.H / in.G);
  float S[RD];
  float* Sp = Sst + (((int64_t)slot * in.H + h) * D) * in.Dv + v0 + col;
#pragma unroll
  for (int i = 0; i < RD; ++i) {
    const int d = rg * RD + i;
    S[i] = (p0 > 0 && d < D && vok) ? Sp[(int64_t)d * in.Dv] : 0.f;
  }
  const AT* qp = in.qk + in.q_off + (int64_t)g * D;
  const AT* kp = in.qk + in.k_off + (int64_t)g * D;
  const AT* zp = in.z + (int64_t)h * D;
  const float rate = DELTA ? in.rate[h] : 0.f;
  const int nblk = (n + LS_TB - 1) / LS_TB;
  // a wave fetches whole rows: rows w, w + 4, ... of the block's 8 x (q, k, decay); lanes over the channels
  float pr[6][NE], pv[2], pb = 0.f;
  auto fetch = [&](int blk) {
    const int64_t t0 = (int64_t)q0 + blk * LS_TB;
    const int nt = min(LS_TB, n - blk * LS_TB);
#pragma unroll
    for (int e = 0; e < 6; ++e) {
      const int row = w + 4 * e, j = row / 3, which = row - 3 * j;
      const AT* src = which == 0 ? qp + (t0 + j) * in.qk_s : which == 1 ? kp + (t0 + j) * in.qk_s : zp + (t0 + j) * in.z_s;
#pragma unroll
      for (int i = 0; i < NE; ++i) {
        const int d = lane + 64 * i;
        pr[e][i] = (j < nt && d < D) ? ldf(src + d) : 0.f;
      }
    }
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const int j = w + 4 * e;
      pv[e] = (j < nt && v0 + lane < in.Dv) ? ldf(in.v + (t0 + j) * in.v_s + (int64_t)h * in.Dv + v0 + lane) : 0.f;
    }
    if (DELTA && threadIdx.x < LS_TB)
      pb = (int)threadIdx.x < nt ? ldf(in.beta + (t0 + threadIdx.x) * in.beta_s + h) : 0.f;
  };
  auto stage = [&](int buf) {
#pragma unroll
    for (int e = 0; e < 6; ++e) {
      const int row = w + 4 * e, j = row / 3, which = row - 3 * j;   // (uniform per wave)
      float sc = which == 0 ? in.qscale : 1.0f;
      if (DELTA && which < 2) {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < NE; ++i) s += pr[e][i] * pr[e][i];
        sc = sc / sqrtf(wave_sum(s) + UNIT_EPS);
      }
#pragma unroll
      for (int i = 0; i < NE; ++i) {
        const int d = lane + 64 * i;
        float v;
        if (which == 2)
          v = d < D ? expf(log_decay<DELTA>(pr[e][i] + in.z_bias[h * D + d], rate, in.inv_tau)) : 1.0f;
        else
          v = pr[e][i] * sc;
        if (d < DMAX) st[buf][j][which][d + 4 * (d / RD)] = v;
      }
    }
#pragma unroll
    for (int e = 0; e < 2; ++e) vs[buf][w + 4 * e][lane] = pv[e];
    if (DELTA && threadIdx.x < LS_TB) bs[buf][threadIdx.x] = sigmoidf(pb);
  };
  if (n > 0) {
    fetch(0);
    stage(0);
  }
  for (int blk = 0; blk < nblk; ++blk) {
    const int buf = blk & 1;
    const int nt = min(LS_TB, n - blk * LS_TB);
    if (blk + 1 < nblk) fetch(blk + 1);
    lds_barrier();   // this block is staged; every wave is done with the other buffer
#pragma unroll 1
    for (int j = 0; j < nt; ++j) {
      const f32x4* qv = reinterpret_cast<const f32x4*>(&st[buf][j][0][rg * (RD + 4)]);
      const f32x4* kv = reinterpret_cast<const f32x4*>(&st[buf][j][1][rg * (RD + 4)]);
      const f32x4* fv = reinterpret_cast<const f32x4*>(&st[buf][j][2][rg * (RD + 4)]);
      float u = vs[buf][j][col];
      if constexpr (DELTA) {
        float d0 = 0.f, d1 = 0.f;
#pragma unroll
        for (int i4 = 0; i4 < RD / 4; ++i4) {
          const f32x4 f4 = fv[i4], k4 = kv[i4];
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[4 * i4 + e] *= f4[e];
            if (e & 1) d1 += S[4 * i4 + e] * k4[e];
            else d0 += S[4 * i4 + e] * k4[e];
          }
        }
        float dot = d0 + d1;
        dot += __shfl_xor(dot, 16, 64);
        dot += __shfl_xor(dot, 32, 64);
        u = bs[buf][j] * (u - dot);
      }
      float o0 = 0.f, o1 = 0.f;
#pragma unroll
      for (int i4 = 0; i4 < RD / 4; ++i4) {
        const f32x4 q4 = qv[i4], k4 = kv[i4];
        f32x4 f4 = {1.f, 1.f, 1.f, 1.f};
        if constexpr (!DELTA) f4 = fv[i4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          float s = S[4 * i4 + e];
          if constexpr (!DELTA) s *= f4[e];
          s += k4[e] * u;
          S[4 * i4 + e] = s;
          if (e & 1) o1 += s * q4[e];
          else o0 += s * q4[e];
        }
      }
      float o = o0 + o1;
      o += __shfl_xor(o, 16, 64);
      o += __shfl_xor(o, 32, 64);
      if (rg == 0 && vok) out[((int64_t)q0 + blk * LS_TB + j) * os + (int64_t)h * in.Dv + v0 + col] = o;
    }
    if (blk + 1 < nblk) stage(buf ^ 1);
  }
#pragma unroll
  for (int i = 0; i < RD; ++i) {
    const int d = rg * RD + i;
    if (d < D && vok) Sp[(int64_t)d * in.Dv] = S[i];
  }
}

// ---- chunks ----------------------------------------------------------------------------------------------------------
constexpr int CH = 32;            // tokens of a chunk: two blocks of 16
constexpr int DS = 64;            // channels of a staged slice
constexpr int LD = DS + 4;        // its LDS row stride
constexpr float FAST_LOG2 = 60.f; // decay of a block (in powers of two) up to which e^(-b) is formed directly
constexpr float MIN_LOG2 = -43.f; // log2 decays of one token are cut off here (2^-43: nothing of the old state is left)

__device__ __forceinline__ f32x4 mfma16f(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
// The wait states a matrix product's result needs before another instruction reads it. The compiler inserts them within
// straight-line code, but was seen to leave them out where a branch lies between the product and the reader: products
// whose results are read behind a branch are kept out of conditional code and followed by this.
__device__ __forceinline__ void mfma_settle() {
  __builtin_amdgcn_sched_barrier(0);
  asm volatile("s_nop 15");
  __builtin_amdgcn_sched_barrier(0);
}

// Scratch of a chunk and head, index ch = chunk H + head (Dp = D rounded up to 16, NV = ceil(Dv / 16)). "Fragments": 16 x
// 16 tiles in the operand layout of the scan's products, [64 lanes][4], lane l holding columns 4 (l / 16) .. + 3 of row
// l % 16 (a lane's four values serve four steps; which of the tile's columns a step takes does not matter as long as
// both operands agree).
struct ChunkBuf {
  float* Q;    // [2][Dp / 16] fragments: rows t, columns d of q_t e^(b_t)
  float* W;    // [2][Dp / 16] fragments: rows t, columns d of W (delta rule)
  float* K;    // [Dp / 16][2] fragments: rows d, columns t of k_t e^(b_end - b_t)
  float* E;    // [Dp]         e^(b_end)
  float* P;    // [32][32]
  float* U;    // [2][NV] tiles of U0 in the accumulator layout: lane l holds rows 4 (l / 16) .. + 3 of column l % 16
};

// out[row m of x][row n of y] over the DS channels of two LDS slices, 16 x 16, channel order permuted alike in both
__device__ __forceinline__ f32x4 block_dot(const float* x, const float* y, int lane, f32x4 acc) {
  const int m = lane & 15, kq = lane >> 4;
#pragma unroll
  for (int s = 0; s < DS / 16; ++s) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(x + m * LD + 16 * s + 4 * kq);
    const f32x4 b = *reinterpret_cast<const f32x4*>(y + m * LD + 16 * s + 4 * kq);
#pragma unroll
    for (int i = 0; i < 4; ++i) acc = mfma16f(a[i], b[i], acc);
  }
  return acc;
}

constexpr int LA = CH + 4;   // LDS row stride of the 32 x 32 matrices

// One workgroup per (chunk, head). Channels go by in NS slices of 64: wave w holds rows 8 w .. 8 w + 7, a lane one
// channel of every slice. e^(b_t - b_j) is split at the start of row t's block of 16 (reference r): e^(b_t - r) <= 1 for
// row t, e^(r - b_j) for key j - also <= 1 for keys of the earlier block; within a block it grows to e^(the block's
// decay), which is formed only while that stays below 2^60. A slice with a faster decay takes its within-block products
// pair by pair. The delta rule's unit lower triangular I + A is inverted by blocks of 16 (forward substitution on the
// diagonal, T21 = -T22 A21 T11); W and U0 are then products with T diag(beta).
template <typename AT, int NS, bool DELTA>
__global__ __launch_bounds__(NT) void lin_chunk_prep_kernel(LinIn<AT> in, const int* __restrict__ vseg, ChunkBuf cb) {
  __shared__ __attribute__((aligned(16))) float qs[CH * LD], kn[CH * LD], kc[16 * LD];
  __shared__ __attribute__((aligned(16))) float ks[(DELTA ? NS : 1) * CH * LD];   // k_t e^(b_t - r), kept for W
  __shared__ __attribute__((aligned(16))) float As[DELTA ? CH * LA : 4];
  __shared__ float Ps[CH * LA];
  __shared__ float tot[4][DS];
  __shared__ __attribute__((aligned(16))) float e1s[NS * DS];   // e^(decay of the first block) per channel
  __shared__ float bt[CH];
  float* Tm = qs;   // the inverse, and the diagonal blocks of A by [key][row]: after the last slice
  float* At = kn;
  const int c = blockIdx.x, h = blockIdx.y;
  const int t0 = vseg[4 * c], n = vseg[4 * c + 1];
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int m = lane & 15, kq = lane >> 4;
  const int D = in.D, Dp = (D + 15) & ~15, ndt = Dp >> 4, g = h / (in.H / in.G);
  const int64_t ch = (int64_t)c * in.H + h;
  const float rate = DELTA ? in.rate[h] : 0.f;
  float* Qo = cb.Q + ch * CH * Dp;
  float* Ko = cb.K + ch * CH * Dp;
  // ---- this thread's inputs, all slices: 8 rows of one channel each
  float qv[NS][8], kv[NS][8], b[NS][8], zb[NS];
  {
    const AT* qp = in.qk + in.q_off + (int64_t)g * D;
    const AT* kp = in.qk + in.k_off + (int64_t)g * D;
    const AT* zp = in.z + (int64_t)h * D;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int t = 8 * w + j;
      const int64_t row = t0 + min(t, n - 1);
      const AT* qr = qp + row * in.qk_s;
      const AT* kr = kp + row * in.qk_s;
      const AT* zr = zp + row * in.z_s;
#pragma unroll
      for (int s = 0; s < NS; ++s) {
        const int d = min(DS * s + lane, D - 1);
        qv[s][j] = ldf(qr + d);
        kv[s][j] = ldf(kr + d);
        b[s][j] = ldf(zr + d);
      }
    }
#pragma unroll
    for (int s = 0; s < NS; ++s) zb[s] = in.z_bias[h * D + min(DS * s + lane, D - 1)];
  }
  if (DELTA && threadIdx.x < CH)
    bt[threadIdx.x] =
        (int)threadIdx.x < n ? sigmoidf(ldf(in.beta + (int64_t)(t0 + threadIdx.x) * in.beta_s + h)) : 0.f;
  for (int i = threadIdx.x; i < CH * LA; i += NT) {
    Ps[i] = 0.f;
    if (DELTA) As[i] = 0.f;
  }
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const bool ok = 8 * w + j < n;
    float sq = 0.f, sk = 0.f;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      if (!ok || DS * s + lane >= D) qv[s][j] = kv[s][j] = 0.f;
      sq += qv[s][j] * qv[s][j];
      sk += kv[s][j] * kv[s][j];
    }
    float fq = in.qscale, fk = 1.0f;
    if (DELTA) {   // unit vectors
      fq = in.qscale / sqrtf(wave_sum(sq) + UNIT_EPS);
      fk = 1.0f / sqrtf(wave_sum(sk) + UNIT_EPS);
    }
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      qv[s][j] *= fq;
      kv[s][j] *= fk;
      const float lg = ok && DS * s + lane < D ? log_decay<DELTA>(b[s][j] + zb[s], rate, in.inv_tau) * LOG2E : 0.f;
      b[s][j] = fmaxf(lg, MIN_LOG2) + (j > 0 ? b[s][j > 0 ? j - 1 : 0] : 0.f);   // running sum over the wave's rows
    }
  }
  const int b0 = w >> 1;   // block of this wave's rows
  f32x4 acc0 = {0, 0, 0, 0}, acc1 = {0, 0, 0, 0};
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    if (DS * s < Dp) {
      const int d = DS * s + lane;
      float* kss = ks + (DELTA ? s * CH * LD : 0);
      __syncthreads();   // (tot and the previous slice's LDS are free)
      tot[w][lane] = b[s][7];
      __syncthreads();
      const float ref1 = tot[0][lane] + tot[1][lane], end1 = tot[2][lane] + tot[3][lane];
      const float before = (w & 1) ? tot[w - 1][lane] : 0.f;                     // rows count from their block's start
      const bool fast = !__any(-ref1 > FAST_LOG2 || -end1 > FAST_LOG2);          // (the same in all waves)
      const float e1 = fast_exp2(ref1);
      const float endl = b0 ? end1 : ref1 + end1;                                // the chunk's end from the block's start
      f32x4 ko[2];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int t = 8 * w + j;
        const float bl = b[s][j] + before;
        b[s][j] = bl;
        const float eb = fast_exp2(bl);
        qs[t * LD + lane] = qv[s][j] * eb;
        if (DELTA) kss[t * LD + lane] = kv[s][j] * eb;
        kn[t * LD + lane] = fast ? kv[s][j] * fast_exp2(-bl) : 0.f;
        if (!b0) kc[t * LD + lane] = kv[s][j] * fast_exp2(ref1 - bl);
        ko[j >> 2][j & 3] = kv[s][j] * fast_exp2(endl - bl);
      }
      if (w == 0) e1s[d] = e1;
      if (d < Dp) {
#pragma unroll
        for (int q4 = 0; q4 < 2; ++q4)   // columns 8 w + 4 q4 .. + 3 of row d
          *reinterpret_cast<f32x4*>(Ko + ((((d >> 4) * 2 + b0) * 64) + (2 * (w & 1) + q4) * 16 + (d & 15)) * 4) = ko[q4];
        if (w == 0) cb.E[ch * Dp + d] = fast_exp2(ref1 + end1);
      }
      __syncthreads();
      // Q fragments of the slice: wave w takes column tile w of both row blocks
      if (DS * s + 16 * w < Dp) {
        const int dt = (DS / 16) * s + w;
        const f32x4 ev = *reinterpret_cast<const f32x4*>(&e1s[16 * dt + 4 * kq]);
#pragma unroll
        for (int rt = 0; rt < 2; ++rt) {
          f32x4 v = *reinterpret_cast<const f32x4*>(qs + (16 * rt + m) * LD + 16 * w + 4 * kq);
          if (rt) v *= ev;
          *reinterpret_cast<f32x4*>(Qo + ((rt * ndt + dt) * 64 + lane) * 4) = v;
        }
      }
      {   // waves 0 / 1: the blocks on the diagonal, waves 2 / 3 (alike): the block below it; P, and A for the delta rule
        const int ro = 16 * min(w, 1) * LD;
        const float* y = w < 2 ? kn + ro : kc;   // (kn is zero in a slice whose pairs are taken one by one)
        acc0 = block_dot(qs + ro, y, lane, acc0);
        if (DELTA) acc1 = block_dot(kss + ro, y, lane, acc1);
        mfma_settle();
      }
      if (!fast) {   // (uniform) pair by pair, from the plain queries, keys and running decays
        __syncthreads();
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const int t = 8 * w + j;
          qs[t * LD + lane] = qv[s][j];
          kss[t * LD + lane] = kv[s][j];
          kn[t * LD + lane] = b[s][j];
        }
        __syncthreads();
        const int tr = threadIdx.x >> 4, kj = threadIdx.x & 15;
        if (kj <= tr) {
          float dp0 = 0.f, dp1 = 0.f, da0 = 0.f, da1 = 0.f;
#pragma unroll 4
          for (int i = 0; i < DS; ++i) {
            const int a = tr * LD + i, k = kj * LD + i;
            const float x0 = kss[k] * fast_exp2(kn[a] - kn[k]);
            const float x1 = kss[k + 16 * LD] * fast_exp2(kn[a + 16 * LD] - kn[k + 16 * LD]);
            dp0 += qs[a] * x0;
            dp1 += qs[a + 16 * LD] * x1;
            da0 += kss[a] * x0;
            da1 += kss[a + 16 * LD] * x1;
          }
          Ps[tr * LA + kj] += dp0;
          Ps[(16 + tr) * LA + 16 + kj] += dp1;
          if (DELTA) {
            As[tr * LA + kj] += da0;
            As[(16 + tr) * LA + 16 + kj] += da1;
          }
        }
        if (DELTA) {   // the decayed keys again, for W
          __syncthreads();
#pragma unroll
          for (int j = 0; j < 8; ++j) kss[(8 * w + j) * LD + lane] = kv[s][j] * fast_exp2(b[s][j]);
        }
      }
    }
  }
  __syncthreads();
  // accumulators -> LDS: waves 0 / 1 the blocks on the diagonal, wave 2 the block below it
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 4 * kq + i;
    if (w < 2) {
      const int o = (16 * w + r) * LA + 16 * w + m;
      Ps[o] = m <= r ? Ps[o] + acc0[i] : 0.f;
      if (DELTA) At[(16 * w + m) * 20 + r] = m < r ? bt[16 * w + r] * (As[o] + acc1[i]) : 0.f;   // [key][row]
    } else if (w == 2) {
      Ps[(16 + r) * LA + m] = acc0[i];
      if (DELTA) As[(16 + r) * LA + m] = bt[16 + r] * acc1[i];
    }
  }
  __syncthreads();
  if (!DELTA || w > 0) {
    for (int i = DELTA ? threadIdx.x - 64 : threadIdx.x; i < CH * CH; i += DELTA ? NT - 64 : NT)
      cb.P[ch * CH * CH + i] = Ps[(i >> 5) * LA + (i & 31)];
  }
  if constexpr (DELTA) {
    if (w == 0) {
      // inverses of the diagonal blocks, a lane per (block, column); lanes 32 .. 63 repeat lanes 0 .. 31
      const int blk = kq & 1;
      float x[16];
#pragma unroll
      for (int t = 0; t < 16; ++t) x[t] = t == m ? 1.0f : 0.f;
#pragma unroll
      for (int j = 0; j < 15; ++j) {
#pragma unroll
        for (int t4 = (j + 1) / 4; t4 < 4; ++t4) {
          const f32x4 a = *reinterpret_cast<const f32x4*>(&At[(16 * blk + j) * 20 + 4 * t4]);
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (4 * t4 + i > j) x[4 * t4 + i] -= a[i] * x[j];
        }
      }
      if (lane < 32) {
#pragma unroll
        for (int t = 0; t < 16; ++t) Tm[(16 * blk + t) * LA + 16 * blk + m] = x[t];
      }
      // T21 = -T22 (A21 T11); the inner product's accumulators are the outer one's right operand
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
      f32x4 u = {0, 0, 0, 0}, v = {0, 0, 0, 0};
      const f32x4 a21 = *reinterpret_cast<const f32x4*>(&As[(16 + m) * LA + 4 * kq]);
      const f32x4 t22 = *reinterpret_cast<const f32x4*>(&Tm[(16 + m) * LA + 16 + 4 * kq]);
#pragma unroll
      for (int i = 0; i < 4; ++i) u = mfma16f(a21[i], Tm[(4 * kq + i) * LA + m], u);
#pragma unroll
      for (int i = 0; i < 4; ++i) v = mfma16f(t22[i], u[i], v);
#pragma unroll
      for (int i = 0; i < 4; ++i) Tm[(16 + 4 * kq + i) * LA + m] = -v[i];
    }
    __syncthreads();
    // T diag(beta): fragments of its three blocks (rows t, columns j)
    f32x4 tf[3];
#pragma unroll
    for (int q = 0; q < 3; ++q) {
      const int r = q ? 16 : 0, j0 = q == 2 ? 16 : 0;
      tf[q] = *reinterpret_cast<const f32x4*>(&Tm[(r + m) * LA + j0 + 4 * kq]);
      const f32x4 bv = {bt[j0 + 4 * kq], bt[j0 + 4 * kq + 1], bt[j0 + 4 * kq + 2], bt[j0 + 4 * kq + 3]};
      tf[q] *= bv;
    }
    float* Wo = cb.W + ch * CH * Dp;
    for (int dt = w; dt < ndt; dt += 4) {   // transposed tiles of W: rows d, columns t
      const float* kb = ks + (dt >> 2) * CH * LD + (dt & 3) * 16 + m;
      const float e1 = e1s[16 * dt + m];
      f32x4 w0 = {0, 0, 0, 0}, w1 = {0, 0, 0, 0};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float k0 = kb[(4 * kq + i) * LD], k1 = kb[(16 + 4 * kq + i) * LD] * e1;
        w0 = mfma16f(k0, tf[0][i], w0);
        w1 = mfma16f(k0, tf[1][i], w1);
        w1 = mfma16f(k1, tf[2][i], w1);
      }
      *reinterpret_cast<f32x4*>(Wo + (dt * 64 + lane) * 4) = w0;
      *reinterpret_cast<f32x4*>(Wo + ((ndt + dt) * 64 + lane) * 4) = w1;
    }
    const int NV = (in.Dv + 15) >> 4;
    float* Uo = cb.U + ch * 2 * NV * 256;
    for (int vt = w; vt < NV; vt += 4) {
      const int vc = min(16 * vt + m, in.Dv - 1);
      const AT* vp = in.v + (int64_t)h * in.Dv + vc;
      float vv[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int t = 16 * (i >> 2) + 4 * kq + (i & 3);
        vv[i] = ldf(vp + (int64_t)(t0 + min(t, n - 1)) * in.v_s);
        if (t >= n || 16 * vt + m >= in.Dv) vv[i] = 0.f;
      }
      f32x4 u0 = {0, 0, 0, 0}, u1 = {0, 0, 0, 0};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        u0 = mfma16f(tf[0][i], vv[i], u0);
        u1 = mfma16f(tf[1][i], vv[i], u1);
        u1 = mfma16f(tf[2][i], vv[4 + i], u1);
      }
      *reinterpret_cast<f32x4*>(Uo + (vt * 64 + lane) * 4) = u0;
      *reinterpret_cast<f32x4*>(Uo + ((NV + vt) * 64 + lane) * 4) = u1;
    }
  }
}

// One workgroup per (16 value columns, head, segment): the D x 16 slice of the state sits in the accumulators of its four
// waves (wave w: row tiles w NTL .. w NTL + NTL - 1; FULL: D = 64 NTL, every wave has all its tiles). An accumulator
// register i of lane l holds row 4 (l / 16) + i, column l % 16 of its tile, which is the right operand of a product over
// the rows {i, 4 + i, 8 + i, 12 + i}: the state enters the products straight from the registers. Per chunk: W S and
// (Q e^b) S over the wave's rows; the waves' parts of W S are summed through LDS to U; the state's update; a quarter of
// P U per wave; the waves' parts of the output summed through LDS. The operands of the next two chunks are in flight.
// The column tiles of a head are given to workgroups of one XCD where the heads divide by 8: they read the same operands.
template <typename AT, int NTL, bool FULL, bool DELTA>
__global__ __launch_bounds__(NT) __attribute__((amdgpu_waves_per_eu(1, NTL > 2 ? 1 : 2))) void lin_chunk_scan_kernel(
    LinIn<AT> in, const int* __restrict__ vseg, const int* __restrict__ cs, ChunkBuf cb, float* __restrict__ Sst,
    float* __restrict__ out, int64_t os) {
  __shared__ f32x4 red[4][2][64];
  __shared__ __attribute__((aligned(16))) f32x4 redo[2][4][2][64];
  const int D = in.D, Dv = in.Dv, Dp = (D + 15) & ~15, NV = (Dv + 15) >> 4, ndt = Dp >> 4;
  int vt, h;
  if (in.H % 8 == 0) {
    const int q = blockIdx.x >> 3;
    vt = q % NV;
    h = (q / NV) * 8 + (blockIdx.x & 7);
  } else {
    vt = blockIdx.x % NV;
    h = blockIdx.x / NV;
  }
  const int r = blockIdx.y;
  const int first = cs[4 * r], cnt = cs[4 * r + 1], p0 = cs[4 * r + 2], slot = cs[4 * r + 3];
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, m = lane & 15, kq = lane >> 4;
  const int vcol = vt * 16 + m;
  float* Sp = Sst + (((int64_t)slot * in.H + h) * D) * Dv + vcol;
  f32x4 S[NTL];
#pragma unroll
  for (int a = 0; a < NTL; ++a)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = (w * NTL + a) * 16 + 4 * kq + i;
      S[a][i] = (p0 > 0 && d < D && vcol < Dv) ? Sp[(int64_t)d * Dv] : 0.f;
    }
  struct Ops {
    f32x4 W[2][NTL], Q[2][NTL], K[NTL][2], E[NTL], U[2];
    f32x2 P[2];
  };
  Ops ops[2];
  // a segment's chunks are consecutive rows, all whole but the last
  const int last = first + cnt, row0 = cnt > 0 ? vseg[4 * first] : 0;
  const int tail = cnt > 0 ? vseg[4 * (last - 1) + 1] : 0;
  // a wave without a tile of its own reads the last tile and holds no state there (its key operand is zeroed): no
  // product is conditional
  auto tile = [&](int a) { return FULL ? w * NTL + a : min(w * NTL + a, ndt - 1); };
  auto load_a = [&](Ops& o, int c) {
    const int64_t ch = (int64_t)c * in.H + h;
    const float* Qp = cb.Q + ch * CH * Dp + lane * 4;
    const float* Wp = DELTA ? cb.W + ch * CH * Dp + lane * 4 : nullptr;
#pragma unroll
    for (int a = 0; a < NTL; ++a)
#pragma unroll
      for (int rt = 0; rt < 2; ++rt) {
        o.Q[rt][a] = *reinterpret_cast<const f32x4*>(Qp + (rt * ndt + tile(a)) * 256);
        if (DELTA) o.W[rt][a] = *reinterpret_cast<const f32x4*>(Wp + (rt * ndt + tile(a)) * 256);
      }
  };
  auto load_b = [&](Ops& o, int c) {
    const int64_t ch = (int64_t)c * in.H + h;
    const float* Kp = cb.K + ch * CH * Dp + lane * 4;
#pragma unroll
    for (int a = 0; a < NTL; ++a) {
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) o.K[a][tt] = *reinterpret_cast<const f32x4*>(Kp + (tile(a) * 2 + tt) * 256);
      o.E[a] = *reinterpret_cast<const f32x4*>(cb.E + ch * Dp + tile(a) * 16 + 4 * kq);
    }
#pragma unroll
    for (int rt = 0; rt < 2; ++rt)
      o.P[rt] = *reinterpret_cast<const f32x2*>(cb.P + ch * CH * CH + (16 * rt + m) * CH + 16 * (w >> 1) + 4 * kq +
                                                2 * (w & 1));
    if constexpr (DELTA) {
#pragma unroll
      for (int tt = 0; tt < 2; ++tt)
        o.U[tt] = *reinterpret_cast<const f32x4*>(cb.U + ((ch * 2 + tt) * NV + vt) * 256 + lane * 4);
    } else {
      const int rows = c + 1 < last ? CH : tail;
      const AT* vp = in.v + (int64_t)(row0 + CH * (c - first)) * in.v_s + (int64_t)h * Dv + min(vcol, Dv - 1);
#pragma unroll
      for (int tt = 0; tt < 2; ++tt)
#pragma unroll
        for (int i = 0; i < 4; ++i) o.U[tt][i] = ldf(vp + (int64_t)min(16 * tt + 4 * kq + i, rows - 1) * in.v_s);
    }
  };
  auto step = [&](Ops& o, int c) {
    f32x4 ws[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}}, ow[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
#pragma unroll
    for (int a = 0; a < NTL; ++a)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int rt = 0; rt < 2; ++rt) {
          if (DELTA) ws[rt] = mfma16f(o.W[rt][a][i], S[a][i], ws[rt]);
          ow[rt] = mfma16f(o.Q[rt][a][i], S[a][i], ow[rt]);
        }
    mfma_settle();
    const int t0 = row0 + CH * (c - first), n = c + 1 < last ? CH : tail;
    if (c + 2 < last) load_a(o, c + 2);
    if constexpr (DELTA) {
      red[w][0][lane] = ws[0];
      red[w][1][lane] = ws[1];
      lds_barrier();
#pragma unroll
      for (int tt = 0; tt < 2; ++tt)
        o.U[tt] -= (red[0][tt][lane] + red[1][tt][lane]) + (red[2][tt][lane] + red[3][tt][lane]);
    } else {
#pragma unroll
      for (int tt = 0; tt < 2; ++tt)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (16 * tt + 4 * kq + i >= n || vcol >= Dv) o.U[tt][i] = 0.f;
    }
    {
      const f32x4 us = (w >> 1) ? o.U[1] : o.U[0];
      const float u0 = (w & 1) ? us[2] : us[0], u1 = (w & 1) ? us[3] : us[1];
#pragma unroll
      for (int rt = 0; rt < 2; ++rt) {
        ow[rt] = mfma16f(o.P[rt][0], u0, ow[rt]);
        ow[rt] = mfma16f(o.P[rt][1], u1, ow[rt]);
      }
    }
    f32x4* ro = &redo[c & 1][0][0][0];
    ro[(w * 2 + 0) * 64 + lane] = ow[0];
    ro[(w * 2 + 1) * 64 + lane] = ow[1];
#pragma unroll
    for (int a = 0; a < NTL; ++a) {
      S[a] *= o.E[a];
#pragma unroll
      for (int tt = 0; tt < 2; ++tt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float k = FULL || w * NTL + a < ndt ? o.K[a][tt][i] : 0.f;
          S[a] = mfma16f(k, o.U[tt][i], S[a]);
        }
    }
    mfma_settle();
    if (c + 2 < last) load_b(o, c + 2);
    lds_barrier();
    {
      const int rt = threadIdx.x >> 7, l2 = (threadIdx.x & 127) >> 1, part = threadIdx.x & 1;
      const f32x2* rp = reinterpret_cast<const f32x2*>(ro) + (rt * 64 + l2) * 2 + part;
      const f32x2 ov = (rp[0] + rp[256]) + (rp[512] + rp[768]);
      const int t = 16 * rt + 4 * (l2 >> 4) + 2 * part, v = vt * 16 + (l2 & 15);
      if (v < Dv) {
        if (t < n) out[(int64_t)(t0 + t) * os + (int64_t)h * Dv + v] = ov[0];
        if (t + 1 < n) out[(int64_t)(t0 + t + 1) * os + (int64_t)h * Dv + v] = ov[1];
      }
    }
  };
#pragma unroll
  for (int k = 0; k < 2; ++k)
    if (k < cnt) {
      load_a(ops[k], first + k);
      load_b(ops[k], first + k);
    }
  for (int c = first; c < last; c += 2) {
    step(ops[0], c);
    if (c + 1 < last) step(ops[1], c + 1);
  }
#pragma unroll
  for (int a = 0; a < NTL; ++a)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = (w * NTL + a) * 16 + 4 * kq + i;
      if (d < D && vcol < Dv) Sp[(int64_t)d * Dv] = S[a][i];
    }
}

// ---- one token per segment -------------------------------------------------------------------------------------------
// Decode steps move the whole state through once: one workgroup per (segment of one row, head, 64 value columns), thread
// (rg, cq) keeps rows rg, 16 + rg, ... of four columns (16-byte loads, 256 contiguous bytes per row). The state's loads are
// issued first; q, k and the decays are staged meanwhile, their norms enter as factors of the products.
template <typename AT, int NR, bool DELTA>
__global__ __launch_bounds__(NT) __attribute__((amdgpu_waves_per_eu(4))) void lin_step_kernel(
    LinIn<AT> in, const int* __restrict__ seg, float* __restrict__ Sst, float* __restrict__ out, int64_t os) {
  __shared__ float qsh[16 * NR], ksh[16 * NR], fsh[16 * NR];
  __shared__ float nrm[2][4];
  __shared__ __attribute__((aligned(16))) float red[2][4][64];
  const int r = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * 64;
  const int q0 = seg[4 * r], n = seg[4 * r + 1], p0 = seg[4 * r + 2], slot = seg[4 * r + 3];
  if (n != 1) return;   // (uniform)
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, rg = tid >> 4, cq = tid & 15;
  const int D = in.D, Dv = in.Dv, g = h / (in.H / in.G);
  const int c4 = v0 + 4 * cq;
  const bool vok = c4 < Dv;
  // (rows and columns past the head's read its last ones: their keys and queries are zero, nothing of them is stored)
  float* Sp = Sst + (((int64_t)slot * in.H + h) * D) * Dv + min(c4, Dv - 4);
  f32x4 S[NR];
  if (p0 > 0) {   // (uniform)
#pragma unroll
    for (int i = 0; i < NR; ++i) S[i] = *reinterpret_cast<const f32x4*>(Sp + min(16 * i + rg, D - 1) * Dv);
  } else {
#pragma unroll
    for (int i = 0; i < NR; ++i) S[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  float vx[4] = {0.f, 0.f, 0.f, 0.f};
  if (vok) {
#pragma unroll
    for (int e = 0; e < 4; ++e) vx[e] = ldf(in.v + (int64_t)q0 * in.v_s + (int64_t)h * Dv + c4 + e);
  }
  const float beta = DELTA ? sigmoidf(ldf(in.beta + (int64_t)q0 * in.beta_s + h)) : 0.f;
  float q = 0.f, k = 0.f;
  if (tid < 16 * NR) {   // (channels past D: q = k = 0, decay 1)
    float f = 1.0f;
    if (tid < D) {
      q = ldf(in.qk + (int64_t)q0 * in.qk_s + in.q_off + (int64_t)g * D + tid);
      k = ldf(in.qk + (int64_t)q0 * in.qk_s + in.k_off + (int64_t)g * D + tid);
      f = expf(log_decay<DELTA>(ldf(in.z + (int64_t)q0 * in.z_s + (int64_t)h * D + tid) + in.z_bias[h * D + tid],
                                DELTA ? in.rate[h] : 0.f, in.inv_tau));
    }
    qsh[tid] = q;
    ksh[tid] = k;
    fsh[tid] = f;
  }
  if (DELTA) {
    const float sq = wave_sum(q * q), sk = wave_sum(k * k);
    if (lane == 0) {
      nrm[0][w] = sq;
      nrm[1][w] = sk;
    }
  }
  lds_barrier();
  float fq = in.qscale, fk = 1.0f;
  if (DELTA) {
    fq = in.qscale / sqrtf((nrm[0][0] + nrm[0][1]) + (nrm[0][2] + nrm[0][3]) + UNIT_EPS);
    fk = 1.0f / sqrtf((nrm[1][0] + nrm[1][1]) + (nrm[1][2] + nrm[1][3]) + UNIT_EPS);
  }
  // sums over all rows of a column: across the wave's four row groups, then across the waves
  auto col_sum = [&](f32x4 v, int buf) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[e] += __shfl_xor(v[e], 16, 64);
      v[e] += __shfl_xor(v[e], 32, 64);
    }
    if (lane < 16) *reinterpret_cast<f32x4*>(&red[buf][w][4 * cq]) = v;
    lds_barrier();
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i) s += *reinterpret_cast<const f32x4*>(&red[buf][i][4 * cq]);
    return s;
  };
  f32x4 u = {vx[0], vx[1], vx[2], vx[3]};
  if constexpr (DELTA) {
    f32x4 dot = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      S[i] *= fsh[16 * i + rg];
      dot += S[i] * ksh[16 * i + rg];
    }
    dot = col_sum(dot, 0);
    u = (u - dot * fk) * (beta * fk);   // (beta (v - S^T k), times the key's norm)
  }
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int d = 16 * i + rg;
    if (!DELTA) S[i] *= fsh[d];
    S[i] += u * ksh[d];
    o += S[i] * qsh[d];
    if (d < D && vok) *reinterpret_cast<f32x4*>(Sp + d * Dv) = S[i];
  }
  o = col_sum(o, 1);
  if (rg == 0 && vok) *reinterpret_cast<f32x4*>(out + (int64_t)q0 * os + (int64_t)h * Dv + c4) = o * fq;
}

static inline int ew_grid(int64_t n) { return (int)std::min<int64_t>((n + 255) / 256, 65535 * 4); }

}  // namespace hl
}  // namespace kafka

using namespace kafka::hl;

#define DISPATCH_AT(f32, ...)             \
  if (f32) {                              \
    using AT = float;                     \
    __VA_ARGS__;                          \
  } else {                                \
    using AT = bf16;                      \
    __VA_ARGS__;                          \
  }

extern "C" {

int kafka_hy_norm_add_max_slabs() { return NA_MAXS; }

hipError_t kafka_hy_norm_add(int f32, float* x, int64_t xs, const void* y1, int64_t y1s, int y1_f32, int S, int64_t slab,
                             const void* y2, int64_t y2s, const float* w, float eps, void* out, int64_t os, int64_t T,
                             int d, hipStream_t st) {
  if (T <= 0 || d <= 0) return hipSuccess;
  if (S < 1 || S > NA_MAXS || (S > 1 && !y1_f32)) return hipErrorInvalidValue;
  auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const bool v4 = d % 4 == 0 && xs % 4 == 0 && y1s % 4 == 0 && slab % 4 == 0 && y2s % 4 == 0 && os % 4 == 0 && al(x) &&
                  al(y1) && al(y2) && al(w) && al(out);
#define NA_LAUNCH(VEC, NV, SL) \
  norm_add_kernel<AT, VEC, NV, SL><<<(unsigned)T, NT, 0, st>>>(x, xs, y1, y1s, slab, (const AT*)y2, y2s, w, eps, (AT*)out, os, d)
#define NA_S(VEC, NV)                         \
  do {                                        \
    if (!y1_f32) NA_LAUNCH(VEC, NV, 0);       \
    else if (S == 1) NA_LAUNCH(VEC, NV, 1);   \
    else if (S == 2) NA_LAUNCH(VEC, NV, 2);   \
    else if (S == 4) NA_LAUNCH(VEC, NV, 4);   \
    else NA_LAUNCH(VEC, NV, 8);               \
  } while (0)
  const bool s8 = !y1_f32 || S == 1 || S == 2 || S == 4 || S == 8;
  DISPATCH_AT(f32, {
    if (v4 && s8 && d <= NT * 4) NA_S(4, 1);
    else if (v4 && s8 && d <= NT * 8) NA_S(4, 2);
    else if (v4 && s8 && d <= NT * 16) NA_S(4, 4);
    else if (v4 && s8 && d <= NT * 32) NA_S(4, 8);
    else if (s8 && d <= NT * 4) NA_S(1, 4);
    else
      norm_add_wide_kernel<AT><<<(unsigned)T, NT, 0, st>>>(x, xs, y1, y1s, y1_f32, S, slab, (const AT*)y2, y2s, w, eps,
                                                           (AT*)out, os, d);
  });
#undef NA_S
#undef NA_LAUNCH
  return hipGetLastError();
}

// glu: out [T, F] = silu(u[:, :F]) * u[:, F:], else out = relu(u)^2
hipError_t kafka_hy_ff_act(int f32, const void* u, int64_t us, void* out, int64_t os, int64_t T, int F, int glu,
                           hipStream_t st) {
  if (T <= 0 || F <= 0) return hipSuccess;
  auto al = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  if (!f32 && F % 8 == 0 && us % 8 == 0 && os % 8 == 0 && al(u) && al(out)) {
    if (glu)
      act_vec8_kernel<true><<<ew_grid(T * (F / 8)), 256, 0, st>>>((const bf16*)u, us, (bf16*)out, os, T, F);
    else
      act_vec8_kernel<false><<<ew_grid(T * (F / 8)), 256, 0, st>>>((const bf16*)u, us, (bf16*)out, os, T, F);
    return hipGetLastError();
  }
  DISPATCH_AT(f32, {
    if (glu) silu_mul_kernel<AT><<<ew_grid(T * F), 256, 0, st>>>((const AT*)u, us, (AT*)out, os, T, F);
    else relu2_kernel<AT><<<ew_grid(T * F), 256, 0, st>>>((const AT*)u, us, (AT*)out, os, T, F);
  });
  return hipGetLastError();
}

int kafka_hy_lin_max_d() { return 256; }
int kafka_hy_lin_chunk() { return CH; }

// rate == nullptr: gated linear attention, else the gated delta rule
hipError_t kafka_hy_lin_scan(int f32, const void* qk, int64_t qk_s, int q_off, int k_off, const void* v, int64_t v_s,
                             const void* z, int64_t z_s, const float* z_bias, const float* rate, const void* beta,
                             int64_t beta_s, int H, int G, int D, int Dv, float qscale, float inv_tau, const int* seg,
                             int R, int min_n, int max_n, float* S, float* out, int64_t os, hipStream_t st) {
  if (R <= 0) return hipSuccess;
  if (D < 1 || D > 256 || Dv < 1 || G < 1 || H % G || H > 65535 || R > 65535 || (rate != nullptr) != (beta != nullptr))
    return hipErrorInvalidValue;
  const dim3 grid((Dv + 63) / 64, H, R);
  // segments of one row: the step kernel, where rows of four columns can be moved in 16-byte pieces
  const bool step = min_n <= 1 && Dv % 4 == 0 && os % 4 == 0 && (reinterpret_cast<uintptr_t>(S) & 15) == 0 &&
                    (reinterpret_cast<uintptr_t>(out) & 15) == 0;
  DISPATCH_AT(f32, {
    const LinIn<AT> in{(const AT*)qk, (const AT*)v, (const AT*)z, (const AT*)beta, z_bias, rate, qk_s, v_s, z_s, beta_s,
                       q_off, k_off, H, G, D, Dv, qscale, inv_tau};
    auto a = [&](auto k) { k<<<grid, NT, 0, st>>>(in, seg, step ? 2 : min_n, max_n, S, out, os); };
    auto a1 = [&](auto k) { k<<<grid, NT, 0, st>>>(in, seg, S, out, os); };
    if (rate != nullptr) {
      if (step) {
        if (D <= 64) a1(lin_step_kernel<AT, 4, true>);
        else if (D <= 128) a1(lin_step_kernel<AT, 8, true>);
        else a1(lin_step_kernel<AT, 16, true>);
      }
      if (max_n > 1 || !step) {
        if (D <= 64) a(lin_scan_kernel<AT, 16, true>);
        else if (D <= 128) a(lin_scan_kernel<AT, 32, true>);
        else a(lin_scan_kernel<AT, 64, true>);
      }
    } else {
      if (step) {
        if (D <= 64) a1(lin_step_kernel<AT, 4, false>);
        else if (D <= 128) a1(lin_step_kernel<AT, 8, false>);
        else a1(lin_step_kernel<AT, 16, false>);
      }
      if (max_n > 1 || !step) {
        if (D <= 64) a(lin_scan_kernel<AT, 16, false>);
        else if (D <= 128) a(lin_scan_kernel<AT, 32, false>);
        else a(lin_scan_kernel<AT, 64, false>);
      }
    }
  });
  return hipGetLastError();
}

// floats of scratch per (chunk, head): Q, K (, W), E, P (, U0)
int64_t kafka_hy_lin_chunk_scratch(int D, int Dv, int delta) {
  const int64_t Dp = (D + 15) & ~15, NV = (Dv + 15) >> 4;
  return (delta ? 3 : 2) * CH * Dp + Dp + CH * CH + (delta ? 2 * NV * 256 : 0);
}

hipError_t kafka_hy_lin_chunked(int f32, const void* qk, int64_t qk_s, int q_off, int k_off, const void* v, int64_t v_s,
                                const void* z, int64_t z_s, const float* z_bias, const float* rate, const void* beta,
                                int64_t beta_s, int H, int G, int D, int Dv, float qscale, float inv_tau,
                                const int* vseg, int n_chunks, const int* cs, int R, float* scratch, float* S,
                                float* out, int64_t os, hipStream_t st) {
  if (R <= 0 || n_chunks <= 0) return hipSuccess;
  if (D < 1 || D > 256 || Dv < 1 || G < 1 || H % G || H > 65535 || R > 65535 ||
      (rate != nullptr) != (beta != nullptr) || (reinterpret_cast<uintptr_t>(scratch) & 15))
    return hipErrorInvalidValue;
  const int64_t Dp = (D + 15) & ~15, NV = (Dv + 15) >> 4, N = (int64_t)n_chunks * H;
  ChunkBuf cb;
  cb.Q = scratch;
  cb.K = cb.Q + N * CH * Dp;
  cb.E = cb.K + N * CH * Dp;
  cb.P = cb.E + N * Dp;
  cb.W = cb.P + N * CH * CH;
  cb.U = cb.W + N * CH * Dp;
  if (rate == nullptr) cb.W = cb.U = nullptr;
  const dim3 g1(n_chunks, H), g2((unsigned)(NV * H), R);
  DISPATCH_AT(f32, {
    const LinIn<AT> in{(const AT*)qk, (const AT*)v, (const AT*)z, (const AT*)beta, z_bias, rate, qk_s, v_s, z_s, beta_s,
                       q_off, k_off, H, G, D, Dv, qscale, inv_tau};
    auto p = [&](auto k) { k<<<g1, NT, 0, st>>>(in, vseg, cb); };
    auto b = [&](auto k) { k<<<g2, NT, 0, st>>>(in, vseg, cs, cb, S, out, os); };
    if (rate != nullptr) {
      if (D <= 64) p(lin_chunk_prep_kernel<AT, 1, true>);
      else if (D <= 128) p(lin_chunk_prep_kernel<AT, 2, true>);
      else p(lin_chunk_prep_kernel<AT, 4, true>);
      if (D == 64) b(lin_chunk_scan_kernel<AT, 1, true, true>);
      else if (D == 128) b(lin_chunk_scan_kernel<AT, 2, true, true>);
      else if (D < 64) b(lin_chunk_scan_kernel<AT, 1, false, true>);
      else if (D < 128) b(lin_chunk_scan_kernel<AT, 2, false, true>);
      else b(lin_chunk_scan_kernel<AT, 4, false, true>);
    } else {
      if (D <= 64) p(lin_chunk_prep_kernel<AT, 1, false>);
      else if (D <= 128) p(lin_chunk_prep_kernel<AT, 2, false>);
      else p(lin_chunk_prep_kernel<AT, 4, false>);
      if (D == 64) b(lin_chunk_scan_kernel<AT, 1, true, false>);
      else if (D == 128) b(lin_chunk_scan_kernel<AT, 2, true, false>);
      else if (D < 64) b(lin_chunk_scan_kernel<AT, 1, false, false>);
      else if (D < 128) b(lin_chunk_scan_kernel<AT, 2, false, false>);
      else b(lin_chunk_scan_kernel<AT, 4, false, false>);
    }
  });
  return hipGetLastError();
}

}  // extern "C"
