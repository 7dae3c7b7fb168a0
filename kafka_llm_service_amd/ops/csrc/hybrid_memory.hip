// Matrix-memory (mLSTM) kernels for single tokens and for long segments, for gfx950.
//
// Per head, with log gates i_t (capped) and f_t <= 0, a running maximum m and q' = q D^(-1/2):
//   m_t = max(f_t + m_(t-1), i_t);  S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(i_t - m_t) k_t v_t^T;  n_t alike with k_t alone;
//   o_t = S_t^T q'_t / (max(|n_t . q'_t|, e^(-m_t)) + 1e-6)
// State, gates and every product with them are fp32 (or as exact as fp32, see below). A step's rows are described by
// segments (seg[r] = first row, rows, first position, state slot); a segment whose first position is 0 starts from zero.
//
//   mlstm_step    segments of one row: one workgroup owns a (segment, head) and moves the memory through registers once in
//                 16-byte pieces
//   mlstm_chunk_* long segments in chunks of 128 tokens (bf16 q, k, v). With F_t the running sum of the chunk's f,
//                 a_t = i_t - F_t, c_t = max_{j <= t} a_j and m0 the running maximum before the chunk:
//                   m_t = F_t + mu_t, mu_t = max(m0, c_t)
//                   S_t^T q_t = e^(m0 - mu_t) S_0^T q_t + sum_{j <= t} e^(a_j - mu_t) (k_j . q_t) v_j
//                 and the chunk's own contribution to the memory, relative to its maximum M = c_end, is
//                   U = sum_j e^(a_j - M) k_j v_j^T;  S' = e^(m0 - mu) S_0 + e^(M - mu) U,  mu = max(m0, M),  m' = F_end + mu
//                 No exponent is positive, whatever the gates.
//     chunk_state   U^T and its normaliser for every chunk in parallel
//     chunk_carry   the chunks' entry states in order (in place of U), the sequence's state advanced
//     chunk_out     the read-outs for every chunk in parallel
//   All products run on the bf16 matrix cores: q, k and v are bf16, the fp32 factor of a product (scaled keys, weights,
//   entry states) is split into three bf16 parts that hold all 24 bits of it, one product each.
#include "common.h"

namespace kafka {
namespace hm {

template <typename T>
__device__ __forceinline__ float ldf(const T* p) { return (float)(*p); }

constexpr int NT = 256;
constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float log_gate(float z, float cap, bool forget) {
  const float c = cap * tanhf(z / cap);
  return forget ? fminf(c, 0.f) - log1pf(expf(-fabsf(c))) : c;   // forget: logsigmoid
}

// ---- one token per segment ------------------------------------------------------------------------------------------
// Thread (rg, cq): rows rg, RG + rg, ... of the four columns at 4 cq; CQ threads across a row.
template <typename AT, int CQ>
__global__ __launch_bounds__(NT) void mlstm_step_kernel(const AT* __restrict__ qkv, int64_t qs,
                                                        const float* __restrict__ gates, int64_t gs, int H, int D,
                                                        int Dv, float cap, const int* __restrict__ seg,
                                                        float* __restrict__ Sst, float* __restrict__ nst,
                                                        float* __restrict__ mst, float* __restrict__ out, int64_t os) {
  constexpr int RG = NT / CQ, NB = 8;
  __shared__ float qsh[256], ksh[256];
  __shared__ float red[NT / 64];
  __shared__ __attribute__((aligned(16))) float osum[NT / 64][4 * CQ];
  const int h = blockIdx.x, r = blockIdx.y;
  const int q0 = seg[4 * r], n = seg[4 * r + 1], p0 = seg[4 * r + 2], slot = seg[4 * r + 3];
  if (n != 1) return;   // (uniform)
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, rg = tid / CQ, cq = tid % CQ;
  const int64_t head = (int64_t)slot * H + h;
  const AT* row = qkv + (int64_t)q0 * qs;
  const float ig = log_gate(gates[(int64_t)q0 * gs + h], cap, false);
  const float fg = log_gate(gates[(int64_t)q0 * gs + H + h], cap, true);
  const float m0 = p0 > 0 ? mst[head] : 0.f;
  const float m = fmaxf(fg + m0, ig), dec = expf(fg + m0 - m), gain = expf(ig - m);
  float nq = 0.f;
  if (tid < 256) {
    float q = 0.f, k = 0.f;
    if (tid < D) {
      q = ldf(row + (int64_t)h * D + tid) / sqrtf((float)D);
      k = ldf(row + (int64_t)(H + h) * D + tid);
      const float nn = dec * (p0 > 0 ? nst[head * D + tid] : 0.f) + gain * k;
      nst[head * D + tid] = nn;
      nq = nn * q;
    }
    qsh[tid] = q;
    ksh[tid] = k;
  }
  nq = block_sum<NT>(nq, red);   // (its barriers also publish q and k, and order the reads of m before its write)
  if (tid == 0) mst[head] = m;
  const float inv = 1.0f / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
  float* Sh = Sst + head * D * Dv;
  for (int cb = 0; cb < Dv; cb += 4 * CQ) {
    const int c4 = cb + 4 * cq;
    const bool vok = c4 < Dv;
    float* Sp = Sh + min(c4, Dv - 4);   // (columns past the head's read its last ones, nothing of them is stored)
    f32x4 v, o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = gain * ldf(row + 2 * (int64_t)H * D + (int64_t)h * Dv + min(c4, Dv - 4) + e);
    for (int d0 = 0; d0 < D; d0 += NB * RG) {
      f32x4 S[NB];
#pragma unroll
      for (int i = 0; i < NB; ++i)
        S[i] = p0 > 0 ? *reinterpret_cast<const f32x4*>(Sp + (int64_t)min(d0 + i * RG + rg, D - 1) * Dv)
                      : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NB; ++i) {
        const int d = d0 + i * RG + rg;
        if (d < D) {
          S[i] = S[i] * dec + v * ksh[d];
          o += S[i] * qsh[d];
          if (vok) *reinterpret_cast<f32x4*>(Sp + (int64_t)d * Dv) = S[i];
        }
      }
    }
#pragma unroll
    for (int x = 32; x >= CQ; x >>= 1)
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] += __shfl_xor(o[e], x, 64);
    __syncthreads();   // (the previous column block's sums have been read)
    if (lane < CQ) *reinterpret_cast<f32x4*>(&osum[w][4 * cq]) = o;
    __syncthreads();
    if (tid < CQ && vok) {
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NT / 64; ++i) s += *reinterpret_cast<const f32x4*>(&osum[i][4 * cq]);
      float* op = out + (int64_t)q0 * os + (int64_t)h * Dv + c4;
#pragma unroll
      for (int e = 0; e < 4; ++e) op[e] = s[e] * inv;
    }
  }
}

// ---- chunks ---------------------------------------------------------------------------------------------------------
constexpr int CH = 128;         // tokens per chunk
constexpr int VSL = 64;         // value columns of a workgroup
constexpr int LDJ = CH + 8;     // row length of a transposed tile in LDS
constexpr int DS = 128;         // key channels staged at a time

struct ChunkIn {
  const bf16* qkv;      // rows [q heads | k heads | v heads]
  int64_t qs;
  const float* gates;   // raw [input | forget]
  int64_t gs;
  int H, D, Dv;
  float cap;
  const int* vseg;      // [chunks][4] = (first row, rows, -, -)
  float* U;             // [chunks][H][Dv][D]: own contribution, then entry state
  float* un;            // [chunks][H][D]: the same for the normaliser
  float* sc;            // [chunks][H][4] = F_end, M, m0
};

// v = a + b + c with bf16 parts that hold all its bits
struct Split {
  bf16x8 p[3];
};
__device__ __forceinline__ Split split3(const float (&v)[8]) {
  Split s;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const bf16 a = (bf16)v[e];
    const float r = v[e] - (float)a;
    const bf16 b = (bf16)r;
    s.p[0][e] = a;
    s.p[1][e] = b;
    s.p[2][e] = (bf16)(r - (float)b);
  }
  return s;
}

// results of matrix products are complete before anything behind a branch reads them
__device__ __forceinline__ void mfma_settle() {
  __builtin_amdgcn_sched_barrier(0);
  asm volatile("s_nop 15");
  __builtin_amdgcn_sched_barrier(0);
}

// which (chunk, head, value slice): a (chunk, head)'s slices run on one XCD (workgroups go round the eight XCDs)
__device__ __forceinline__ bool chunk_item(int items, int slices, int& item, int& slice) {
  const int lin = blockIdx.x, xcd = lin & 7, k = lin >> 3;
  item = (k / slices) * 8 + xcd;
  slice = k % slices;
  return item < items;
}
__host__ __device__ __forceinline__ int chunk_grid(int items, int slices) { return (items + 7) / 8 * 8 * slices; }

// The chunk's gates by one wave: a_t, its running maximum c_t and F_t to LDS (rows past n: f = 0, a = -inf).
__device__ __forceinline__ void chunk_gates(const ChunkIn& in, int row0, int n, int h, int lane, float* a_s, float* c_s,
                                            float* F_s) {
  float f[2], g[2];
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    const int t = 64 * k + lane;
    f[k] = 0.f;
    g[k] = -INFINITY;
    if (t < n) {
      const float* z = in.gates + (int64_t)(row0 + t) * in.gs + h;
      g[k] = log_gate(z[0], in.cap, false);
      f[k] = log_gate(z[in.H], in.cap, true);
    }
  }
#pragma unroll
  for (int k = 0; k < 2; ++k)
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float u = __shfl_up(f[k], o, 64);
      if (lane >= o) f[k] += u;
    }
  f[1] += __shfl(f[0], 63, 64);
  float c[2];
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    c[k] = g[k] - f[k];
    a_s[64 * k + lane] = c[k];
    F_s[64 * k + lane] = f[k];
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float u = __shfl_up(c[k], o, 64);
      if (lane >= o) c[k] = fmaxf(c[k], u);
    }
  }
  c[1] = fmaxf(c[1], __shfl(c[0], 63, 64));
#pragma unroll
  for (int k = 0; k < 2; ++k) c_s[64 * k + lane] = c[k];
}

// rows row0 .. row0 + 127 (past n: the last one), columns c0 .. c0 + nc - 1 of the head's part at col -> tile[column][row]
__device__ __forceinline__ void stage_transposed(const bf16* src, int64_t stride, int n, int c0, int nc, int ncols,
                                                 bf16* tile, int tid) {
  const int cgs = nc >> 3;
  for (int u = tid; u < cgs * (CH / 4); u += NT) {
    const int cg = u % cgs, rq = u / cgs, c = c0 + 8 * cg;
    bf16x8 x[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      x[k] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
      if (c < ncols) x[k] = load_bf16x8(src + (int64_t)min(4 * rq + k, n - 1) * stride + c);
    }
    typedef bf16 bf16x4 __attribute__((ext_vector_type(4)));
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const bf16x4 y = {x[0][e], x[1][e], x[2][e], x[3][e]};
      *reinterpret_cast<bf16x4*>(tile + (8 * cg + e) * LDJ + 4 * rq) = y;
    }
  }
}

__global__ __launch_bounds__(NT) void mlstm_chunk_state_kernel(ChunkIn in, int n_chunks, int slices) {
  __shared__ __attribute__((aligned(16))) bf16 Kt[DS * LDJ];
  __shared__ __attribute__((aligned(16))) bf16 Vt[VSL * LDJ];
  __shared__ float a_s[CH], c_s[CH], F_s[CH];
  int item, slice;
  if (!chunk_item(n_chunks * in.H, slices, item, slice)) return;   // (uniform)
  const int ch = item / in.H, h = item - ch * in.H, v0 = slice * VSL;
  const int row0 = in.vseg[4 * ch], n = in.vseg[4 * ch + 1];
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, lr = lane & 31, lh = lane >> 5;
  const int D = in.D, Dv = in.Dv, H = in.H;
  const bf16* rows = in.qkv + (int64_t)row0 * in.qs;
  if (w == 0) chunk_gates(in, row0, n, h, lane, a_s, c_s, F_s);
  stage_transposed(rows + 2 * (int64_t)H * D + (int64_t)h * Dv, in.qs, n, v0, VSL, Dv, Vt, tid);
  for (int db = 0; db < D; db += DS) {
    if (db) __syncthreads();
    stage_transposed(rows + (int64_t)(H + h) * D, in.qs, n, db, min(DS, D - db), D, Kt, tid);
    __syncthreads();
    const float M = c_s[CH - 1];
    const int d = 32 * w + lr;   // (of this block; waves and lanes past D compute on what LDS holds and store nothing)
    f32x16 acc[2];
    float ns = 0.f;
#pragma unroll
    for (int vt = 0; vt < 2; ++vt)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[vt][i] = 0.f;
#pragma unroll 2
    for (int ks = 0; ks < CH / 16; ++ks) {
      const int j = 16 * ks + 8 * lh;
      const bf16x8 kv = *reinterpret_cast<const bf16x8*>(Kt + d * LDJ + j);
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        x[e] = fast_exp2((a_s[j + e] - M) * LOG2E) * (float)kv[e];   // (rows past n: a = -inf, factor 0)
        ns += x[e];
      }
      const Split s = split3(x);
#pragma unroll
      for (int vt = 0; vt < 2; ++vt) {
        const bf16x8 vf = *reinterpret_cast<const bf16x8*>(Vt + (32 * vt + lr) * LDJ + j);
#pragma unroll
        for (int k = 0; k < 3; ++k) acc[vt] = mfma32(vf, s.p[k], acc[vt]);
      }
    }
    mfma_settle();
    ns += __shfl_xor(ns, 32, 64);
    if (db + d < D) {
      float* Up = in.U + ((int64_t)item * Dv + v0) * D + db + d;
#pragma unroll
      for (int vt = 0; vt < 2; ++vt)
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const int v = 32 * vt + (i & 3) + 8 * (i >> 2) + 4 * lh;
          if (v0 + v < Dv) Up[(int64_t)v * D] = acc[vt][i];
        }
      if (slice == 0 && lh == 0) in.un[(int64_t)item * D + db + d] = ns;
    }
  }
  if (slice == 0 && tid == 0) {
    in.sc[4 * (int64_t)item] = F_s[CH - 1];
    in.sc[4 * (int64_t)item + 1] = c_s[CH - 1];
  }
}

// grid (element blocks of Dv * D (+ one block of the normaliser and the maximum), H, segments): cs[r] = (first chunk,
// chunks, first position, state slot)
__global__ __launch_bounds__(NT) void mlstm_chunk_carry_kernel(ChunkIn in, const int* __restrict__ cs,
                                                               float* __restrict__ Sst, float* __restrict__ nst,
                                                               float* __restrict__ mst) {
  const int r = blockIdx.z, h = blockIdx.y, D = in.D, Dv = in.Dv, H = in.H;
  const int first = cs[4 * r], last = first + cs[4 * r + 1], p0 = cs[4 * r + 2], slot = cs[4 * r + 3];
  const int64_t head = (int64_t)slot * H + h;
  // (the block of the normaliser is the only writer of m; the others read it before: it writes m to sc and mlstm_commit
  // stores it in the end)
  float m = p0 > 0 ? mst[head] : 0.f;
  const bool norm = blockIdx.x + 1 == gridDim.x;
  float* st;
  float* el;
  int64_t step;
  if (norm) {
    if ((int)threadIdx.x >= D) return;
    st = nst + head * D + threadIdx.x;
    el = in.un + (int64_t)h * D + threadIdx.x;
    step = (int64_t)H * D;
  } else {
    const int64_t i = (int64_t)blockIdx.x * NT + threadIdx.x;   // element v * D + d
    if (i >= (int64_t)Dv * D) return;
    const int v = (int)(i / D), d = (int)(i - (int64_t)v * D);
    st = Sst + head * D * Dv + (int64_t)d * Dv + v;
    el = in.U + (int64_t)h * Dv * D + i;
    step = (int64_t)H * Dv * D;
  }
  float S = p0 > 0 ? *st : 0.f;
  constexpr int PF = 4;
  float u[PF];
#pragma unroll
  for (int k = 0; k < PF; ++k) u[k] = first + k < last ? el[(int64_t)(first + k) * step] : 0.f;
  for (int c0 = first; c0 < last; c0 += PF) {
    float nx[PF];
#pragma unroll
    for (int k = 0; k < PF; ++k) nx[k] = c0 + PF + k < last ? el[(int64_t)(c0 + PF + k) * step] : 0.f;
#pragma unroll
    for (int k = 0; k < PF; ++k) {
      const int c = c0 + k;
      if (c < last) {
        const float* sc = in.sc + 4 * ((int64_t)c * H + h);
        const float F = sc[0], M = sc[1], mu = fmaxf(m, M);
        el[(int64_t)c * step] = S;                       // the chunk's entry state
        if (norm && threadIdx.x == 0) in.sc[4 * ((int64_t)c * H + h) + 2] = m;
        S = expf(m - mu) * S + expf(M - mu) * u[k];
        m = F + mu;
      }
    }
#pragma unroll
    for (int k = 0; k < PF; ++k) u[k] = nx[k];
  }
  *st = S;
  if (norm && threadIdx.x == 0) in.sc[4 * ((int64_t)(last - 1) * H + h) + 3] = m;
}

// NKS: 16-channel steps of a head held in registers (D <= 16 NKS; the steps past D multiply by zero queries)
template <int NKS>
__global__ __launch_bounds__(NT) void mlstm_chunk_out_kernel(ChunkIn in, const int* __restrict__ cs, int n_segs,
                                                             float* __restrict__ mst, int n_chunks, int slices,
                                                             float* __restrict__ out, int64_t os) {
  // one buffer, first for the entry state's three parts [3][VSL][DS + 8], then for the values [VSL][LDJ]
  constexpr int LDD = DS + 8;
  __shared__ __attribute__((aligned(16))) bf16 buf[3 * VSL * LDD];
  __shared__ float a_s[CH], c_s[CH], F_s[CH], n_s[256];
  // the sequences' maxima: read by every block of the carry kernel, written only now
  for (int i = blockIdx.x * NT + threadIdx.x; i < n_segs * in.H; i += gridDim.x * NT) {
    const int r = i / in.H, h = i - r * in.H;
    mst[(int64_t)cs[4 * r + 3] * in.H + h] = in.sc[4 * ((int64_t)(cs[4 * r] + cs[4 * r + 1] - 1) * in.H + h) + 3];
  }
  int item, slice;
  if (!chunk_item(n_chunks * in.H, slices, item, slice)) return;   // (uniform)
  const int ch = item / in.H, h = item - ch * in.H, v0 = slice * VSL;
  const int row0 = in.vseg[4 * ch], n = in.vseg[4 * ch + 1];
  const int tid = threadIdx.x, w = tid >> 6, lane = tid & 63, lr = lane & 31, lh = lane >> 5;
  const int D = in.D, Dv = in.Dv, H = in.H, nks = D >> 4;
  const bf16* rows = in.qkv + (int64_t)row0 * in.qs;
  const float m0 = in.sc[4 * (int64_t)item + 2];
  if (w == 0) chunk_gates(in, row0, n, h, lane, a_s, c_s, F_s);
  for (int d = tid; d < D; d += NT) n_s[d] = in.un[(int64_t)item * D + d];
  const int t = 32 * w + lr;                       // this lane's row
  const bf16* qrow = rows + (int64_t)min(t, n - 1) * in.qs + (int64_t)h * D + 8 * lh;
  bf16x8 qf[NKS], kf[NKS];
  auto fetch_keys = [&](int jt) {
    const bf16* krow = rows + (int64_t)min(32 * jt + lr, n - 1) * in.qs + (int64_t)(H + h) * D + 8 * lh;
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks) kf[ks] = load_bf16x8(krow + 16 * min(ks, nks - 1));
  };
#pragma unroll
  for (int ks = 0; ks < NKS; ++ks) {
    qf[ks] = load_bf16x8(qrow + 16 * min(ks, nks - 1));
    if (ks >= nks) qf[ks] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
  }
  fetch_keys(0);
  f32x16 acc[2];
#pragma unroll
  for (int vt = 0; vt < 2; ++vt)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[vt][i] = 0.f;
  float nq = 0.f;
  // ---- the entry state: acc = S_0^T q
  for (int db = 0; db < D; db += DS) {
    const int nd = min(DS, D - db), d4s = nd >> 2;
    if (db) __syncthreads();
    for (int u = tid; u < VSL * d4s; u += NT) {
      const int v = u / d4s, d = 4 * (u - v * d4s);
      f32x4 x = {0.f, 0.f, 0.f, 0.f};
      if (v0 + v < Dv) x = *reinterpret_cast<const f32x4*>(in.U + ((int64_t)item * Dv + v0 + v) * D + db + d);
      typedef bf16 bf16x4 __attribute__((ext_vector_type(4)));
      bf16x4 p[3];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const bf16 a = (bf16)x[e];
        const float rr = x[e] - (float)a;
        const bf16 b = (bf16)rr;
        p[0][e] = a;
        p[1][e] = b;
        p[2][e] = (bf16)(rr - (float)b);
      }
#pragma unroll
      for (int k = 0; k < 3; ++k) *reinterpret_cast<bf16x4*>(buf + (k * VSL + v) * LDD + d) = p[k];
    }
    __syncthreads();
    if (32 * w < n) {   // (uniform per wave)
#pragma unroll
      for (int ks = 0; ks < NKS; ++ks) {
        const int d = 16 * ks - db;   // (uniform) the step's channels in this block
        if (d >= 0 && d < nd) {
#pragma unroll
          for (int e = 0; e < 8; ++e) nq += n_s[db + d + 8 * lh + e] * (float)qf[ks][e];
#pragma unroll
          for (int vt = 0; vt < 2; ++vt)
#pragma unroll
            for (int k = 0; k < 3; ++k)
              acc[vt] = mfma32(*reinterpret_cast<const bf16x8*>(buf + (k * VSL + 32 * vt + lr) * LDD + d + 8 * lh),
                               qf[ks], acc[vt]);
        }
      }
      mfma_settle();
    }
  }
  __syncthreads();
  stage_transposed(rows + 2 * (int64_t)H * D + (int64_t)h * Dv, in.qs, n, v0, VSL, Dv, buf, tid);
  __syncthreads();
  if (32 * w >= n) return;   // (uniform per wave; no barrier follows)
  const float mu = fmaxf(m0, c_s[t]);
  const float g0 = fast_exp2((m0 - mu) * LOG2E);
#pragma unroll
  for (int vt = 0; vt < 2; ++vt)
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[vt][i] *= g0;
  nq *= g0;
  // ---- the chunk's own rows: 32 keys at a time, P^T = K q^T (this lane's row: column), its weights split for V^T P^T
  for (int jt = 0; jt <= w; ++jt) {
    f32x16 P;
#pragma unroll
    for (int i = 0; i < 16; ++i) P[i] = 0.f;
#pragma unroll
    for (int ks = 0; ks < NKS; ++ks) P = mfma32(kf[ks], qf[ks], P);
    mfma_settle();
    if (jt < w) fetch_keys(jt + 1);
    float wt[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int j = 32 * jt + (i & 3) + 8 * (i >> 2) + 4 * lh;
      wt[i] = j <= t ? P[i] * fast_exp2((a_s[j] - mu) * LOG2E) : 0.f;   // (rows past n: a = -inf)
      nq += wt[i];
    }
#pragma unroll
    for (int s = 0; s < 2; ++s) {   // 16 keys: this half's are 4 lh .. + 3 and 8 + 4 lh .. + 3
      const float x[8] = {wt[8 * s], wt[8 * s + 1], wt[8 * s + 2], wt[8 * s + 3],
                          wt[8 * s + 4], wt[8 * s + 5], wt[8 * s + 6], wt[8 * s + 7]};
      const Split sp = split3(x);
#pragma unroll
      for (int vt = 0; vt < 2; ++vt) {
        typedef bf16 bf16x4 __attribute__((ext_vector_type(4)));
        const bf16* vp = buf + (32 * vt + lr) * LDJ + 32 * jt + 16 * s + 4 * lh;
        const bf16x4 lo = *reinterpret_cast<const bf16x4*>(vp), hi = *reinterpret_cast<const bf16x4*>(vp + 8);
        const bf16x8 vf = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
#pragma unroll
        for (int k = 0; k < 3; ++k) acc[vt] = mfma32(vf, sp.p[k], acc[vt]);
      }
    }
  }
  mfma_settle();
  nq += __shfl_xor(nq, 32, 64);   // the halves hold different channels and keys
  if (t >= n) return;
  const float qscale = 1.0f / sqrtf((float)D);
  const float inv = qscale / (fmaxf(fabsf(nq * qscale), expf(-(F_s[t] + mu))) + 1e-6f);
  float* op = out + (int64_t)(row0 + t) * os + (int64_t)h * Dv + v0;
#pragma unroll
  for (int vt = 0; vt < 2; ++vt)
#pragma unroll
    for (int i4 = 0; i4 < 4; ++i4) {
      const int v = 32 * vt + 8 * i4 + 4 * lh;
      if (v0 + v < Dv) {
        const f32x4 o = {acc[vt][4 * i4] * inv, acc[vt][4 * i4 + 1] * inv, acc[vt][4 * i4 + 2] * inv,
                         acc[vt][4 * i4 + 3] * inv};
        *reinterpret_cast<f32x4*>(op + v) = o;
      }
    }
}

}  // namespace hm
}  // namespace kafka

using namespace kafka::hm;

extern "C" {

// segments of one row; value sizes that are multiples of 4 (16-byte pieces of the memory's rows)
int kafka_hy_mlstm_step_ok(int D, int Dv) { return D >= 1 && D <= 256 && Dv >= 4 && Dv % 4 == 0; }

hipError_t kafka_hy_mlstm_step(int f32, const void* qkv, int64_t qs, const float* gates, int64_t gs, int H, int D,
                               int Dv, float cap, const int* seg, int R, float* S, float* nrm, float* mx, float* out,
                               int64_t os, hipStream_t st) {
  if (R <= 0) return hipSuccess;
  if (!kafka_hy_mlstm_step_ok(D, Dv) || R > 65535) return hipErrorInvalidValue;
  const dim3 grid(H, R);
#define MS_LAUNCH(AT, CQ)                                                                                            \
  mlstm_step_kernel<AT, CQ><<<grid, NT, 0, st>>>((const AT*)qkv, qs, gates, gs, H, D, Dv, cap, seg, S, nrm, mx, out, os)
#define MS_CQ(AT)                             \
  do {                                        \
    if (Dv <= 32) MS_LAUNCH(AT, 8);           \
    else if (Dv <= 64) MS_LAUNCH(AT, 16);     \
    else if (Dv <= 128) MS_LAUNCH(AT, 32);    \
    else MS_LAUNCH(AT, 64);                   \
  } while (0)
  if (f32) MS_CQ(float); else MS_CQ(bf16);
#undef MS_CQ
#undef MS_LAUNCH
  return hipGetLastError();
}

int kafka_hy_mlstm_chunk() { return CH; }
// bf16 rows whose heads start at multiples of 8 elements
int kafka_hy_mlstm_chunk_ok(int H, int D, int Dv, int64_t qs) {
  return D >= 16 && D % 16 == 0 && D <= 256 && Dv >= 8 && Dv % 8 == 0 && qs % 8 == 0;
}
// floats of scratch per (chunk, head)
int64_t kafka_hy_mlstm_chunk_scratch(int D, int Dv) { return (int64_t)D * Dv + D + 4; }

// the segments of cs in chunks (vseg: all their chunks in order)
hipError_t kafka_hy_mlstm_chunked(const void* qkv, int64_t qs, const float* gates, int64_t gs, int H, int D, int Dv,
                                  float cap, const int* vseg, int n_chunks, const int* cs, int R, float* scratch,
                                  float* S, float* nrm, float* mx, float* out, int64_t os, hipStream_t st) {
  if (R <= 0 || n_chunks <= 0) return hipSuccess;
  if (!kafka_hy_mlstm_chunk_ok(H, D, Dv, qs) || R > 65535 || H > 65535 || os % 4) return hipErrorInvalidValue;
  const int64_t items = (int64_t)n_chunks * H;
  const int slices = (Dv + VSL - 1) / VSL;
  if ((items + 8) * slices > 0x7fffffff) return hipErrorInvalidValue;
  ChunkIn in{(const bf16*)qkv, qs, gates, gs, H, D, Dv, cap, vseg, scratch, scratch + items * D * Dv,
             scratch + items * ((int64_t)D * Dv + D)};
  const unsigned g = (unsigned)chunk_grid((int)items, slices);
  mlstm_chunk_state_kernel<<<g, NT, 0, st>>>(in, n_chunks, slices);
  const dim3 gc((unsigned)(((int64_t)D * Dv + NT - 1) / NT + 1), H, R);
  mlstm_chunk_carry_kernel<<<gc, NT, 0, st>>>(in, cs, S, nrm, mx);
  if (D <= 64) mlstm_chunk_out_kernel<4><<<g, NT, 0, st>>>(in, cs, R, mx, n_chunks, slices, out, os);
  else if (D <= 128) mlstm_chunk_out_kernel<8><<<g, NT, 0, st>>>(in, cs, R, mx, n_chunks, slices, out, os);
  else mlstm_chunk_out_kernel<16><<<g, NT, 0, st>>>(in, cs, R, mx, n_chunks, slices, out, os);
  return hipGetLastError();
}

}  // extern "C"
