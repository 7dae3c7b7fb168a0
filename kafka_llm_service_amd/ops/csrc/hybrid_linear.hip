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
//   lin_chunk_prep / lin_chunk_scan   long segments in chunks of 32 tokens. With b_t the running sum of the chunk's log
//                decays, the chunk's outputs and its new state are matrix products:
//                  P[t][j] = q_t . (k_j e^(b_t - b_j)) (j <= t),  A[t][j] = beta_t k_t . (k_j e^(b_t - b_j)) (j < t)
//                  U = V,  or for the delta rule  (I + A) U = diag(beta) (V - (K e^b) S), i.e. U = U0 - W S with
//                  (I + A) [W | U0] = diag(beta) [K e^b | V] (forward substitution)
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
// load of the row is in flight before the statistics, the sublayer's output and the residual stay in registers.
template <typename AT, int VEC, int NV>
__global__ __launch_bounds__(NT) void norm_add_kernel(float* __restrict__ x, int64_t xs, const void* __restrict__ y1,
                                                      int64_t y1s, int y1_f32, int S, int64_t slab,
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
      if (y1_f32) {
        const float* p = reinterpret_cast<const float*>(y1) + t * y1s + i;
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
__global__ __launch_bounds__(NT) void lin_scan_kernel(LinIn<AT> in, const int* __restrict__ seg, int max_n,
                                                      float* __restrict__ Sst, float* __restrict__ out, int64_t os) {
  constexpr int DMAX = 4 * RD;
  constexpr int LROW = DMAX + 16;            // a row group's rows are shifted by 4 floats: reads of the groups spread
  constexpr int NE = (DMAX + 63) / 64;       // elements of a staged row per lane
  __shared__ __attribute__((aligned(16))) float st[2][LS_TB][3][LROW];   // q, k, decay
  __shared__ float vs[2][LS_TB][64];
  __shared__ float bs[2][LS_TB];
  const int r = blockIdx.z, h = blockIdx.y, v0 = blockIdx.x * 64;
  const int q0 = seg[4 * r], n = seg[4 * r + 1], p0 = seg[4 * r + 2], slot = seg[4 * r + 3];
  if (n > max_n) return;   // (uniform) a segment that the chunk kernels take
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63, rg = lane >> 4;
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

// Scratch of a chunk and head, index ch = chunk H + head (Dp = D rounded up to 16, NV = ceil(Dv / 16)):
struct ChunkBuf {
  float* Q;    // [32][Dp]     q_t e^(b_t)
  float* W;    // [32][Dp]     delta rule: rows of W
  float* K;    // [Dp][32]     k_t e^(b_end - b_t), channel-major
  float* E;    // [Dp]         e^(b_end)
  float* P;    // [32][32]
  float* U;    // [2][NV][64][4]  delta rule: U0 in the accumulator layout of the scan
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

// One workgroup per (chunk, head). Channels go by in slices of 64: wave w holds rows 8 w .. 8 w + 7, a lane one channel.
// e^(b_t - b_j) is split at the start of row t's block (reference r): e^(b_t - r) <= 1 for row t, e^(r - b_j) for key j -
// also <= 1 for keys of an earlier block; within a block it grows to e^(the block's decay), which is formed only while
// that stays below 2^60. A slice with a faster decay takes its within-block products pair by pair.
template <typename AT, bool DELTA>
__global__ __launch_bounds__(NT) void lin_chunk_prep_kernel(LinIn<AT> in, const int* __restrict__ vseg, ChunkBuf cb) {
  __shared__ __attribute__((aligned(16))) float qs[CH * LD], ks[CH * LD], kn[CH * LD], kc[16 * LD];
  __shared__ __attribute__((aligned(16))) float As[CH * 36];
  __shared__ float Ps[CH * 36];
  __shared__ float tot[4][DS];
  __shared__ float rq[CH], rk[CH], bt[CH];
  const int c = blockIdx.x, h = blockIdx.y;
  const int t0 = vseg[4 * c], n = vseg[4 * c + 1];
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int D = in.D, Dp = (D + 15) & ~15, g = h / (in.H / in.G);
  const int64_t ch = (int64_t)c * in.H + h;
  const AT* qp = in.qk + in.q_off + (int64_t)g * D;
  const AT* kp = in.qk + in.k_off + (int64_t)g * D;
  const AT* zp = in.z + (int64_t)h * D;
  const float rate = DELTA ? in.rate[h] : 0.f;
  float* Qo = cb.Q + ch * CH * Dp;
  float* Ko = cb.K + ch * CH * Dp;
  float* Wo = DELTA ? cb.W + ch * CH * Dp : nullptr;
  for (int i = threadIdx.x; i < CH * 36; i += NT) As[i] = Ps[i] = 0.f;
  if (DELTA) {
#pragma unroll
    for (int j = 0; j < 8; ++j) {   // unit norms of this wave's rows
      const int t = 8 * w + j;
      float sq = 0.f, sk = 0.f;
      if (t < n)
        for (int d = lane; d < D; d += 64) {
          const float a = ldf(qp + (int64_t)(t0 + t) * in.qk_s + d), b = ldf(kp + (int64_t)(t0 + t) * in.qk_s + d);
          sq += a * a;
          sk += b * b;
        }
      sq = wave_sum(sq);
      sk = wave_sum(sk);
      if (lane == 0) {
        rq[t] = in.qscale / sqrtf(sq + UNIT_EPS);
        rk[t] = 1.0f / sqrtf(sk + UNIT_EPS);
        bt[t] = t < n ? sigmoidf(ldf(in.beta + (int64_t)(t0 + t) * in.beta_s + h)) : 0.f;
      }
    }
  }
  __syncthreads();
  const int b0 = w < 2 ? 0 : 1;      // block of this wave's rows
  f32x4 acc0 = {0, 0, 0, 0}, acc1 = {0, 0, 0, 0};
  float dp0 = 0.f, dp1 = 0.f, da0 = 0.f, da1 = 0.f;   // pairwise sums of thread (row tid / 16, key tid % 16) per block
  for (int d0 = 0; d0 < Dp; d0 += DS) {
    const int d = d0 + lane;
    float b[8], qv[8], kv[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int t = 8 * w + j;
      const bool ok = t < n && d < D;
      const int64_t row = t0 + (t < n ? t : 0);
      qv[j] = ok ? ldf(qp + row * in.qk_s + d) : 0.f;
      kv[j] = ok ? ldf(kp + row * in.qk_s + d) : 0.f;
      b[j] = ok ? ldf(zp + row * in.z_s + d) : 0.f;
    }
    const float zb = d < D ? in.z_bias[h * D + d] : 0.f;
    float run = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int t = 8 * w + j;
      qv[j] *= DELTA ? rq[t] : in.qscale;
      if (DELTA) kv[j] *= rk[t];
      const float lg = (t < n && d < D) ? log_decay<DELTA>(b[j] + zb, rate, in.inv_tau) * LOG2E : 0.f;
      run += fmaxf(lg, MIN_LOG2);
      b[j] = run;
    }
    tot[w][lane] = run;
    __syncthreads();
    const float ref1 = tot[0][lane] + tot[1][lane], bend = ref1 + (tot[2][lane] + tot[3][lane]);
    // rows of the later block are counted from its start
    const float before = (w & 1) ? tot[w - 1][lane] : 0.f;
    const bool fast = !__any(-ref1 > FAST_LOG2 || ref1 - bend > FAST_LOG2);   // (same in all waves)
    const float e1 = fast_exp2(ref1);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int t = 8 * w + j;
      const float bl = b[j] + before;                      // decay since the block's start
      const float eb = fast_exp2(bl);
      const float full = b0 ? eb * e1 : eb;                // e^(b_t)
      b[j] = bl;
      qs[t * LD + lane] = qv[j] * eb;
      if (DELTA) ks[t * LD + lane] = kv[j] * eb;
      kn[t * LD + lane] = fast ? kv[j] * fast_exp2(-bl) : 0.f;
      if (!b0) kc[t * LD + lane] = kv[j] * fast_exp2(ref1 - bl);
      if (d < Dp) {
        Qo[(int64_t)t * Dp + d] = qv[j] * full;
        if (DELTA) Wo[(int64_t)t * Dp + d] = bt[t] * kv[j] * full;
      }
    }
    if (d < Dp) {
      const float endl = b0 ? bend - ref1 : bend;   // decay up to the chunk's end, from this block's start
#pragma unroll
      for (int q4 = 0; q4 < 2; ++q4) {
        f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = kv[4 * q4 + i] * fast_exp2(endl - b[4 * q4 + i]);
        *reinterpret_cast<f32x4*>(Ko + (int64_t)d * CH + 8 * w + 4 * q4) = v;
      }
      if (w == 0) cb.E[ch * Dp + d] = fast_exp2(bend);
    }
    __syncthreads();
    if (w == 2) {
      acc0 = block_dot(qs + 16 * LD, kc, lane, acc0);
    } else if (w == 3) {
      if (DELTA) acc0 = block_dot(ks + 16 * LD, kc, lane, acc0);
    } else if (fast) {
      acc0 = block_dot(qs + 16 * w * LD, kn + 16 * w * LD, lane, acc0);
      if (DELTA) acc1 = block_dot(ks + 16 * w * LD, kn + 16 * w * LD, lane, acc1);
    }
    if (!fast) {   // (uniform) pair by pair, from the plain queries, keys and running decays
      __syncthreads();
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int t = 8 * w + j;
        qs[t * LD + lane] = qv[j];
        ks[t * LD + lane] = kv[j];
        kn[t * LD + lane] = b[j];
      }
      __syncthreads();
      const int tr = threadIdx.x >> 4, kj = threadIdx.x & 15;
      if (kj <= tr) {
        for (int i = 0; i < DS; ++i) {
          const int a = tr * LD + i, k = kj * LD + i;
          const float x0 = ks[k] * fast_exp2(kn[a] - kn[k]);
          const float x1 = ks[k + 16 * LD] * fast_exp2(kn[a + 16 * LD] - kn[k + 16 * LD]);
          dp0 += qs[a] * x0;
          dp1 += qs[a + 16 * LD] * x1;
          da0 += ks[a] * x0;
          da1 += ks[a + 16 * LD] * x1;
        }
      }
    }
    __syncthreads();   // the slice's LDS is free again
  }
  // accumulators -> LDS: wave 0 / 1 the blocks on the diagonal (P, A), wave 2 / 3 the block below it (P / A)
  {
    const int cc = lane & 15, r0 = 4 * (lane >> 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (w < 2) {
        Ps[(16 * w + r0 + i) * 36 + 16 * w + cc] = acc0[i];
        As[(16 * w + r0 + i) * 36 + 16 * w + cc] = acc1[i];
      } else if (w == 2) {
        Ps[(16 + r0 + i) * 36 + cc] = acc0[i];
      } else {
        As[(16 + r0 + i) * 36 + cc] = acc0[i];
      }
    }
  }
  __syncthreads();
  {
    const int tr = threadIdx.x >> 4, kj = threadIdx.x & 15;
    Ps[tr * 36 + kj] += dp0;
    Ps[(16 + tr) * 36 + 16 + kj] += dp1;
    As[tr * 36 + kj] += da0;
    As[(16 + tr) * 36 + 16 + kj] += da1;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < CH * CH; i += NT) {
    const int t = i / CH, j = i - t * CH;
    cb.P[ch * CH * CH + i] = j <= t ? Ps[t * 36 + j] : 0.f;
    if (DELTA) As[t * 36 + j] = j < t ? bt[t] * As[t * 36 + j] : 0.f;
  }
  if constexpr (DELTA) {
    __syncthreads();   // (also: this workgroup's stores of beta k e^b are visible to its threads)
    // (I + A) X = right-hand side, a thread per column: the channels of W, then the value columns
    const int NV = (in.Dv + 15) >> 4;
    for (int col = threadIdx.x; col < Dp + 16 * NV; col += NT) {
      float x[CH];
      const int vc = col - Dp;
#pragma unroll
      for (int t = 0; t < CH; ++t) {
        if (col < Dp)
          x[t] = Wo[(int64_t)t * Dp + col];
        else
          x[t] = (t < n && vc < in.Dv) ? bt[t] * ldf(in.v + (int64_t)(t0 + t) * in.v_s + (int64_t)h * in.Dv + vc) : 0.f;
      }
#pragma unroll
      for (int t = 1; t < CH; ++t) {
        float s0 = 0.f, s1 = 0.f;
#pragma unroll
        for (int j4 = 0; j4 < (t + 3) / 4; ++j4) {
          const f32x4 a = *reinterpret_cast<const f32x4*>(&As[t * 36 + 4 * j4]);   // (zeros from j = t on)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            if (4 * j4 + i < t) {
              if (i & 1) s1 += a[i] * x[4 * j4 + i];
              else s0 += a[i] * x[4 * j4 + i];
            }
          }
        }
        x[t] -= s0 + s1;
        __builtin_amdgcn_sched_barrier(0);   // (row by row: all of A's rows in flight would not fit the registers)
      }
      if (col < Dp) {
#pragma unroll
        for (int t = 0; t < CH; ++t) Wo[(int64_t)t * Dp + col] = x[t];
      } else {
        float* Uo = cb.U + (ch * 2 * NV + (vc >> 4)) * 256 + (vc & 15) * 4;
#pragma unroll
        for (int q = 0; q < CH / 4; ++q) {
          const f32x4 v = {x[4 * q], x[4 * q + 1], x[4 * q + 2], x[4 * q + 3]};
          *reinterpret_cast<f32x4*>(Uo + (int64_t)(q >> 2) * NV * 256 + (q & 3) * 64) = v;
        }
      }
    }
  }
}

// One workgroup per (16 value columns, head, segment): the D x 16 slice of the state sits in the accumulators of its four
// waves (wave w: row tiles w NTL .. w NTL + NTL - 1). An accumulator register i of lane l holds row 4 (l / 16) + i,
// column l % 16 of its tile, which is the right operand of a product over the rows {i, 4 + i, 8 + i, 12 + i}: the
// state enters the products straight from the registers. Per chunk: W S and (Q e^b) S over the wave's rows; the
// waves' parts of W S are summed through LDS to U; the state's update; a quarter of P U per wave; the waves' parts of
// the output summed through LDS. The next chunk's operands are loaded meanwhile.
template <typename AT, int NTL, bool DELTA>
__global__ __launch_bounds__(NT) void lin_chunk_scan_kernel(LinIn<AT> in, const int* __restrict__ vseg,
                                                            const int* __restrict__ cs, ChunkBuf cb,
                                                            float* __restrict__ Sst, float* __restrict__ out,
                                                            int64_t os) {
  __shared__ f32x4 red[4][2][64];
  __shared__ __attribute__((aligned(16))) f32x4 redo[2][4][2][64];
  const int vt = blockIdx.x, h = blockIdx.y, r = blockIdx.z;
  const int first = cs[4 * r], cnt = cs[4 * r + 1], p0 = cs[4 * r + 2], slot = cs[4 * r + 3];
  const int w = threadIdx.x >> 6, lane = threadIdx.x & 63, m = lane & 15, kq = lane >> 4;
  const int D = in.D, Dv = in.Dv, Dp = (D + 15) & ~15, NV = (Dv + 15) >> 4, ndt = Dp >> 4;
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
  f32x4 Wr[2][NTL], Qr[2][NTL], Kr[NTL][2], Er[NTL], U[2];
  f32x2 Pr[2];
  auto load_a = [&](int c) {
    const int64_t ch = (int64_t)c * in.H + h;
#pragma unroll
    for (int a = 0; a < NTL; ++a) {
      const int dt = w * NTL + a;
      if (dt < ndt) {   // (uniform per wave)
#pragma unroll
        for (int rt = 0; rt < 2; ++rt) {
          const int64_t o = (ch * CH + 16 * rt + m) * Dp + dt * 16 + 4 * kq;
          Qr[rt][a] = *reinterpret_cast<const f32x4*>(cb.Q + o);
          if (DELTA) Wr[rt][a] = *reinterpret_cast<const f32x4*>(cb.W + o);
        }
      }
    }
  };
  auto load_b = [&](int c) {
    const int64_t ch = (int64_t)c * in.H + h;
#pragma unroll
    for (int a = 0; a < NTL; ++a) {
      const int dt = w * NTL + a;
      if (dt < ndt) {
#pragma unroll
        for (int tt = 0; tt < 2; ++tt)
          Kr[a][tt] = *reinterpret_cast<const f32x4*>(cb.K + (ch * Dp + dt * 16 + m) * CH + 16 * tt + 4 * kq);
        Er[a] = *reinterpret_cast<const f32x4*>(cb.E + ch * Dp + dt * 16 + 4 * kq);
      }
    }
#pragma unroll
    for (int rt = 0; rt < 2; ++rt)
      Pr[rt] = *reinterpret_cast<const f32x2*>(cb.P + ch * CH * CH + (16 * rt + m) * CH + 16 * (w >> 1) + 4 * kq + 2 * (w & 1));
    if constexpr (DELTA) {
#pragma unroll
      for (int tt = 0; tt < 2; ++tt)
        U[tt] = *reinterpret_cast<const f32x4*>(cb.U + ((ch * 2 + tt) * NV + vt) * 256 + lane * 4);
    } else {
      const int t0 = vseg[4 * c], n = vseg[4 * c + 1];
#pragma unroll
      for (int tt = 0; tt < 2; ++tt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 16 * tt + 4 * kq + i;
          U[tt][i] = (t < n && vcol < Dv) ? ldf(in.v + (int64_t)(t0 + t) * in.v_s + (int64_t)h * Dv + vcol) : 0.f;
        }
    }
  };
  if (cnt > 0) {
    load_a(first);
    load_b(first);
  }
  for (int c = first; c < first + cnt; ++c) {
    f32x4 ws[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}}, ow[2] = {{0, 0, 0, 0}, {0, 0, 0, 0}};
#pragma unroll
    for (int a = 0; a < NTL; ++a) {
      if (w * NTL + a < ndt) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
#pragma unroll
          for (int rt = 0; rt < 2; ++rt) {
            if (DELTA) ws[rt] = mfma16f(Wr[rt][a][i], S[a][i], ws[rt]);
            ow[rt] = mfma16f(Qr[rt][a][i], S[a][i], ow[rt]);
          }
        }
      }
    }
    if (c + 1 < first + cnt) load_a(c + 1);
    if constexpr (DELTA) {
      red[w][0][lane] = ws[0];
      red[w][1][lane] = ws[1];
      lds_barrier();
#pragma unroll
      for (int tt = 0; tt < 2; ++tt)
        U[tt] -= (red[0][tt][lane] + red[1][tt][lane]) + (red[2][tt][lane] + red[3][tt][lane]);
    }
    {
      const f32x4 us = (w >> 1) ? U[1] : U[0];
      const float u0 = (w & 1) ? us[2] : us[0], u1 = (w & 1) ? us[3] : us[1];
#pragma unroll
      for (int rt = 0; rt < 2; ++rt) {
        ow[rt] = mfma16f(Pr[rt][0], u0, ow[rt]);
        ow[rt] = mfma16f(Pr[rt][1], u1, ow[rt]);
      }
    }
    f32x4* ro = &redo[c & 1][0][0][0];
    ro[(w * 2 + 0) * 64 + lane] = ow[0];
    ro[(w * 2 + 1) * 64 + lane] = ow[1];
#pragma unroll
    for (int a = 0; a < NTL; ++a)
      if (w * NTL + a < ndt) S[a] *= Er[a];
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int a = 0; a < NTL; ++a)
          if (w * NTL + a < ndt) S[a] = mfma16f(Kr[a][tt][i], U[tt][i], S[a]);
    const int t0 = vseg[4 * c], n = vseg[4 * c + 1];
    if (c + 1 < first + cnt) load_b(c + 1);
    lds_barrier();
    {
      const int rt = threadIdx.x >> 7, l2 = (threadIdx.x & 127) >> 1, part = threadIdx.x & 1;
      const f32x2* rp = reinterpret_cast<const f32x2*>(ro) + (rt * 64 + l2) * 2 + part;
      const f32x2 o = (rp[0] + rp[256]) + (rp[512] + rp[768]);
      const int t = 16 * rt + 4 * (l2 >> 4) + 2 * part, v = vt * 16 + (l2 & 15);
      if (v < Dv) {
        if (t < n) out[(int64_t)(t0 + t) * os + (int64_t)h * Dv + v] = o[0];
        if (t + 1 < n) out[(int64_t)(t0 + t + 1) * os + (int64_t)h * Dv + v] = o[1];
      }
    }
  }
#pragma unroll
  for (int a = 0; a < NTL; ++a)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = (w * NTL + a) * 16 + 4 * kq + i;
      if (d < D && vcol < Dv) Sp[(int64_t)d * Dv] = S[a][i];
    }
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
  DISPATCH_AT(f32, {
    auto a = [&](auto k) {
      k<<<(unsigned)T, NT, 0, st>>>(x, xs, y1, y1s, y1_f32, S, slab, (const AT*)y2, y2s, w, eps, (AT*)out, os, d);
    };
    if (v4 && d <= NT * 4) a(norm_add_kernel<AT, 4, 1>);
    else if (v4 && d <= NT * 8) a(norm_add_kernel<AT, 4, 2>);
    else if (v4 && d <= NT * 16) a(norm_add_kernel<AT, 4, 4>);
    else if (v4 && d <= NT * 32) a(norm_add_kernel<AT, 4, 8>);
    else if (d <= NT * 4) a(norm_add_kernel<AT, 1, 4>);
    else a(norm_add_wide_kernel<AT>);
  });
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
                             int R, int max_n, float* S, float* out, int64_t os, hipStream_t st) {
  if (R <= 0) return hipSuccess;
  if (D < 1 || D > 256 || Dv < 1 || G < 1 || H % G || H > 65535 || R > 65535 || (rate != nullptr) != (beta != nullptr))
    return hipErrorInvalidValue;
  const dim3 grid((Dv + 63) / 64, H, R);
  DISPATCH_AT(f32, {
    const LinIn<AT> in{(const AT*)qk, (const AT*)v, (const AT*)z, (const AT*)beta, z_bias, rate, qk_s, v_s, z_s, beta_s,
                       q_off, k_off, H, G, D, Dv, qscale, inv_tau};
    auto a = [&](auto k) { k<<<grid, NT, 0, st>>>(in, seg, max_n, S, out, os); };
    if (rate != nullptr) {
      if (D <= 64) a(lin_scan_kernel<AT, 16, true>);
      else if (D <= 128) a(lin_scan_kernel<AT, 32, true>);
      else a(lin_scan_kernel<AT, 64, true>);
    } else {
      if (D <= 64) a(lin_scan_kernel<AT, 16, false>);
      else if (D <= 128) a(lin_scan_kernel<AT, 32, false>);
      else a(lin_scan_kernel<AT, 64, false>);
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
  const dim3 g1(n_chunks, H), g2((unsigned)NV, H, R);
  DISPATCH_AT(f32, {
    const LinIn<AT> in{(const AT*)qk, (const AT*)v, (const AT*)z, (const AT*)beta, z_bias, rate, qk_s, v_s, z_s, beta_s,
                       q_off, k_off, H, G, D, Dv, qscale, inv_tau};
    auto b = [&](auto k) { k<<<g2, NT, 0, st>>>(in, vseg, cs, cb, S, out, os); };
    if (rate != nullptr) {
      lin_chunk_prep_kernel<AT, true><<<g1, NT, 0, st>>>(in, vseg, cb);
      if (D <= 64) b(lin_chunk_scan_kernel<AT, 1, true>);
      else if (D <= 128) b(lin_chunk_scan_kernel<AT, 2, true>);
      else b(lin_chunk_scan_kernel<AT, 4, true>);
    } else {
      lin_chunk_prep_kernel<AT, false><<<g1, NT, 0, st>>>(in, vseg, cb);
      if (D <= 64) b(lin_chunk_scan_kernel<AT, 1, false>);
      else if (D <= 128) b(lin_chunk_scan_kernel<AT, 2, false>);
      else b(lin_chunk_scan_kernel<AT, 4, false>);
    }
  });
  return hipGetLastError();
}

}  // extern "C"
