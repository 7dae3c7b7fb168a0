// Expert products of long steps on wave-tiled expert weights, and what surrounds them, for gfx950.
//
//   grouped_wide   Y = X_e W_e^T per expert segment of the routed entries, 128 rows x 256 columns a workgroup, for steps
//                  whose experts have many rows. The weights come in the wave-tiled order of the weight-streaming
//                  kernels (Wt[E][N/32][K/16][64][8]): a wave owns 64 columns and loads its operands straight from
//                  memory in 1 KB pieces; only the activations go through LDS (64-deep steps, double buffered, next
//                  step's loads in flight), where all four waves share them. Work items are ordered row tile first, then
//                  column tile, then expert, and every XCD takes one contiguous stretch of them: the row tiles of a
//                  column tile run side by side on one L2 and its weights leave memory once.
//                  Epilogues: silu(gate) * up or its clamped form on GLU-interleaved tiles (a wave holds both tiles of a
//                  pair), relu squared, the weighted combine into fp32 rows, or the weighted rows as they are (in entry
//                  order; their consumer gathers a token's rows through the sort's inverse, no atomics).
//   moe_sort       stable sort of (token, choice) entries by expert, one workgroup: every wave counts and then places
//                  its stretch of the entries 64 at a time, equal experts found by ballots over the bits of their ids
//   narrow         fp32 products of bf16 rows with up to 64 bf16 weight rows (router logits, gate projections): 16 rows a
//                  workgroup, its 16 (or 8) waves split K, 16x16x32 products; with a bias, or followed in place by the
//                  choice of the k largest scores, a wave per row
#include "common.h"

namespace kafka {
namespace mw {

// ---- grouped products -------------------------------------------------------------------------------------------------
constexpr int BM = 128, BN = 256, BK = 64;
constexpr int KS = BK / 16;        // matrix steps per staged block
constexpr int MT = BM / 32;        // row tiles
constexpr int XL = BM * (BK / 8) / 256;

enum { EPI_GLU = 0, EPI_RELU2 = 1, EPI_COMBINE = 2, EPI_ROWS = 3 };

// 16-byte piece c (0 .. 7) of LDS row r
__device__ __forceinline__ int xoff(int r, int c) { return r * BK + 8 * (c ^ (r & 7)); }

// item -> (expert, row tile, column tile) over the experts' segments; false past the last item. Every wave does this.
__device__ __forceinline__ bool find_item(const int* expert_off, int E, int ntn, int& e, int& rt, int& nt) {
  const int lane = threadIdx.x & 63;
  // all items, in waves of 64 experts: the total first, then this workgroup's place
  int total = 0;
  for (int b = 0; b < E; b += 64) {
    int t = 0;
    if (b + lane < E) t = (expert_off[b + lane + 1] - expert_off[b + lane] + BM - 1) / BM * ntn;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) t += __shfl_xor(t, o, 64);
    total += t;
  }
  const int per = (total + 7) >> 3, k = blockIdx.x >> 3;
  const int item = (blockIdx.x & 7) * per + k;
  if (k >= per || item >= total) return false;
  int base = 0;
  for (int b = 0; b < E; b += 64) {
    int t = 0;
    if (b + lane < E) t = (expert_off[b + lane + 1] - expert_off[b + lane] + BM - 1) / BM * ntn;
    int incl = t;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int u = __shfl_up(incl, o, 64);
      if (lane >= o) incl += u;
    }
    const unsigned long long hit = __ballot(base + incl > item);
    if (hit) {
      const int l = __builtin_ctzll(hit);
      const int before = base + __shfl(incl - t, l, 64), tiles = __shfl(t, l, 64) / ntn;
      e = __builtin_amdgcn_readfirstlane(b + l);
      const int i = __builtin_amdgcn_readfirstlane(item - before), ti = __builtin_amdgcn_readfirstlane(tiles);
      nt = i / ti;
      rt = i - nt * ti;
      return true;
    }
    base += __shfl(incl, 63, 64);
  }
  return false;
}

template <bool GATHER, int EPI>
__global__ __launch_bounds__(256, 2) void grouped_wide_kernel(const bf16* __restrict__ X, int64_t ldx,
                                                              const bf16x8* __restrict__ Wt, int E, int N, int K,
                                                              const int* __restrict__ perm_tok,
                                                              const float* __restrict__ perm_w,
                                                              const int* __restrict__ expert_off,
                                                              bf16* __restrict__ Y, int64_t ldy,
                                                              float* __restrict__ out, int64_t ldo, float glu_limit,
                                                              float glu_alpha) {
  __shared__ __attribute__((aligned(16))) bf16 xs[2][BM * BK];
  int e, rt, nt;
  if (!find_item(expert_off, E, (N + BN - 1) / BN, e, rt, nt)) return;   // (uniform)
  const int seg0 = expert_off[e] + rt * BM, rows = min(BM, expert_off[e + 1] - seg0);
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, r = lane & 31, h = lane >> 5;
  const int nb = (nt * 4 + w) * 2;                 // this wave's two 32-column tiles
  const bool active = nb < (N >> 5);               // (N is a multiple of 64: both or none)
  const bf16x8* wp = Wt + ((int64_t)e * (N >> 5) + (active ? nb : 0)) * (K >> 4) * 64 + lane;
  const int64_t wstep = (int64_t)(K >> 4) * 64;    // the second tile
  const int nk = K / BK;
  const bf16* xsrc[XL];
  int xdst[XL];
#pragma unroll
  for (int i = 0; i < XL; ++i) {
    const int idx = tid + 256 * i, row = idx >> 3, c = idx & 7;
    const int ent = seg0 + min(row, rows - 1);     // rows past the segment reload a valid row, never stored
    xsrc[i] = X + (GATHER ? (int64_t)perm_tok[ent] : (int64_t)ent) * ldx + c * 8;
    xdst[i] = xoff(row, c);
  }
  bf16x8 xr[XL], wa[KS][2], wb[KS][2];
  auto load_x = [&](int ch) {
#pragma unroll
    for (int i = 0; i < XL; ++i) xr[i] = load_bf16x8(xsrc[i] + ch * BK);
  };
  auto store_x = [&](int buf) {
#pragma unroll
    for (int i = 0; i < XL; ++i) *reinterpret_cast<bf16x8*>(&xs[buf][xdst[i]]) = xr[i];
  };
  auto load_w = [&](bf16x8(&wv)[KS][2], int ch) {
#pragma unroll
    for (int t = 0; t < KS; ++t)
#pragma unroll
      for (int j = 0; j < 2; ++j) wv[t][j] = wp[(int64_t)(ch * KS + t) * 64 + j * wstep];
    __builtin_amdgcn_sched_barrier(0);             // (requested before this step's products)
  };
  f32x16 acc[MT][2];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[mt][j][i] = 0.f;
  auto compute = [&](int buf, const bf16x8(&wv)[KS][2]) {
#pragma unroll
    for (int t = 0; t < KS; ++t)
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) {
        const bf16x8 xf = *reinterpret_cast<const bf16x8*>(&xs[buf][xoff(mt * 32 + r, 2 * t + h)]);
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[mt][j] = mfma32(xf, wv[t][j], acc[mt][j]);
      }
  };
  load_x(0);
  load_w(wa, 0);
  store_x(0);
  __syncthreads();
  for (int ch = 0; ch < nk; ch += 2) {               // (nk is even; the last step's prefetch repeats a block)
    load_x(ch + 1);
    load_w(wb, ch + 1);
    compute(0, wa);
    store_x(1);
    __syncthreads();
    const int nx = min(ch + 2, nk - 1);
    load_x(nx);
    load_w(wa, nx);
    compute(1, wb);
    store_x(0);
    __syncthreads();
  }
  // the last products' results are complete before anything reads them behind a branch
  __builtin_amdgcn_sched_barrier(0);
  asm volatile("s_nop 15");
  __builtin_amdgcn_sched_barrier(0);
  if (!active) return;
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int m = mt * 32 + (i & 3) + 8 * (i >> 2) + 4 * h;
      if (m >= rows) continue;
      const int ent = seg0 + m;
      if constexpr (EPI == EPI_COMBINE) {
        float* o = out + (int64_t)perm_tok[ent] * ldo + nb * 32 + r;
        const float pw = perm_w[ent];
        atomicAdd(o, pw * acc[mt][0][i]);
        atomicAdd(o + 32, pw * acc[mt][1][i]);
      } else if constexpr (EPI == EPI_ROWS) {
        bf16* y = Y + (int64_t)ent * ldy + nb * 32 + r;
        const float pw = perm_w[ent];
        y[0] = (bf16)(pw * acc[mt][0][i]);
        y[32] = (bf16)(pw * acc[mt][1][i]);
      } else if constexpr (EPI == EPI_RELU2) {
        bf16* y = Y + (int64_t)ent * ldy + nb * 32 + r;
        const float a = fmaxf(acc[mt][0][i], 0.f), b = fmaxf(acc[mt][1][i], 0.f);
        y[0] = (bf16)(a * a);
        y[32] = (bf16)(b * b);
      } else {
        float g = acc[mt][0][i], u = acc[mt][1][i], al = 1.0f;
        if (glu_limit > 0.f) {   // (uniform) the clamped form
          g = fminf(g, glu_limit);
          u = fminf(fmaxf(u, -glu_limit), glu_limit) + 1.0f;
          al = glu_alpha;
        }
        Y[(int64_t)ent * ldy + (nb >> 1) * 32 + r] = (bf16)(g / (1.0f + __expf(-al * g)) * u);
      }
    }
}

// ---- stable sort by expert --------------------------------------------------------------------------------------------
constexpr int SORT_NT = 1024, SORT_W = SORT_NT / 64;
constexpr int SORT_MAXE = 512;

// lanes of the wave whose (valid) entry has this lane's expert
__device__ __forceinline__ unsigned long long same_expert(int e, bool valid, int bits) {
  unsigned long long m = __ballot(valid);
  for (int b = 0; b < bits; ++b) {
    const unsigned long long s = __ballot((e >> b) & 1);
    m &= ((e >> b) & 1) ? s : ~s;
  }
  return m;
}

__global__ __launch_bounds__(SORT_NT) void moe_sort_kernel(const float* __restrict__ topk_w,
                                                           const int* __restrict__ topk_e, int n, int k, int E, int bits,
                                                           int bm, int* __restrict__ perm_tok,
                                                           float* __restrict__ perm_w, int* __restrict__ expert_off,
                                                           int* __restrict__ tile_off, int* __restrict__ inv) {
  __shared__ int cnt[SORT_W][SORT_MAXE];
  __shared__ int sum[2][SORT_W];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  for (int i = tid; i < SORT_W * E; i += SORT_NT) cnt[i / E][i % E] = 0;
  const int per = ((n + SORT_W - 1) / SORT_W + 63) / 64 * 64;   // a wave's stretch of the entries
  const int i0 = w * per, i1 = min(n, i0 + per);
  constexpr int PF = 8;
  __syncthreads();
  for (int b0 = i0; b0 < i1; b0 += 64 * PF) {
    int ev[PF];
#pragma unroll
    for (int p = 0; p < PF; ++p) {
      const int i = b0 + 64 * p + lane;
      ev[p] = i < i1 ? topk_e[i] : 0;
    }
#pragma unroll
    for (int p = 0; p < PF; ++p) {
      const bool valid = b0 + 64 * p + lane < i1;
      const unsigned long long m = same_expert(ev[p], valid, bits);
      if (valid && __builtin_ctzll(m) == lane) cnt[w][ev[p]] += __builtin_popcountll(m);
      __builtin_amdgcn_wave_barrier();
    }
  }
  __syncthreads();
  // per expert: counts -> exclusive sums over the waves; then exclusive sums over the experts (and their row tiles)
  int tot = 0;
  if (tid < E)
    for (int i = 0; i < SORT_W; ++i) {
      const int c = cnt[i][tid];
      cnt[i][tid] = tot;
      tot += c;
    }
  int a = tid < E ? tot : 0, t = tid < E ? (tot + bm - 1) / bm : 0;
  const int a0 = a;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const int u = __shfl_up(a, o, 64), v = __shfl_up(t, o, 64);
    if (lane >= o) {
      a += u;
      t += v;
    }
  }
  if (lane == 63) {
    sum[0][w] = a;
    sum[1][w] = t;
  }
  __syncthreads();
  for (int i = 0; i < w; ++i) {
    a += sum[0][i];
    t += sum[1][i];
  }
  if (tid < E) {
    expert_off[tid + 1] = a;
    tile_off[tid + 1] = t;
    for (int i = 0; i < SORT_W; ++i) cnt[i][tid] += a - a0;
    if (tid == 0) expert_off[0] = tile_off[0] = 0;
  }
  __syncthreads();
  for (int b0 = i0; b0 < i1; b0 += 64 * PF) {
    int ev[PF];
    float wv[PF];
#pragma unroll
    for (int p = 0; p < PF; ++p) {
      const int i = b0 + 64 * p + lane;
      ev[p] = i < i1 ? topk_e[i] : 0;
      wv[p] = i < i1 ? topk_w[i] : 0.f;
    }
#pragma unroll
    for (int p = 0; p < PF; ++p) {
      const int i = b0 + 64 * p + lane;
      const bool valid = i < i1;
      const unsigned long long m = same_expert(ev[p], valid, bits);
      const int at = valid ? cnt[w][ev[p]] : 0;
      __builtin_amdgcn_wave_barrier();             // (every lane has read before the first of an expert moves it on)
      if (valid) {
        const int pos = at + __builtin_popcountll(m & ((1ull << lane) - 1));
        perm_tok[pos] = i / k;
        perm_w[pos] = wv[p];
        if (inv != nullptr) inv[i] = pos;
        if (__builtin_ctzll(m) == lane) cnt[w][ev[p]] = at + __builtin_popcountll(m);
      }
      __builtin_amdgcn_wave_barrier();
    }
  }
}

// ---- narrow products --------------------------------------------------------------------------------------------------
constexpr int NR_ROWS = 16, NR_MAXN = 64, NR_MAXK = 16;
// waves of a workgroup and row length of their parts in LDS, TN: tiles of 16 weight rows
__host__ __device__ constexpr int nr_waves(int TN) { return TN <= 2 ? 16 : 8; }
__host__ __device__ constexpr int nr_ld(int TN) { return 16 * TN + 1; }
typedef float f32x4v __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4v mfma16(bf16x8 a, bf16x8 b, f32x4v c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

// z[row][n] = x[row] . w[n] for 16 rows, the waves' parts summed through LDS -> z in part[0]
template <int TN>
__device__ __forceinline__ void narrow_product(const bf16* __restrict__ x, int64_t xs, int64_t T, const bf16* __restrict__ wt,
                                               int N, int K, float (*part)[NR_ROWS][nr_ld(TN)]) {
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, r = lane & 15, q = lane >> 4;
  const int64_t t = min((int64_t)blockIdx.x * NR_ROWS + r, T - 1);
  const bf16* xp = x + t * xs + 8 * q;
  const bf16* wp[TN];
#pragma unroll
  for (int j = 0; j < TN; ++j) wp[j] = wt + (int64_t)min(16 * j + r, N - 1) * K + 8 * q;
  f32x4v acc[TN];
#pragma unroll
  for (int j = 0; j < TN; ++j) acc[j] = f32x4v{0.f, 0.f, 0.f, 0.f};
  constexpr int PF = TN <= 2 ? 8 : 4;              // steps in flight
  const int ns = K / 32;
  constexpr int NW = nr_waves(TN);
  for (int s0 = w * PF; s0 < ns; s0 += NW * PF) {
    bf16x8 a[PF], b[PF][TN];
#pragma unroll
    for (int p = 0; p < PF; ++p) {
      const int s = min(s0 + p, ns - 1);
      a[p] = load_bf16x8(xp + 32 * s);
      if (s0 + p >= ns) a[p] = bf16x8{0, 0, 0, 0, 0, 0, 0, 0};
#pragma unroll
      for (int j = 0; j < TN; ++j) b[p][j] = load_bf16x8(wp[j] + 32 * s);
    }
#pragma unroll
    for (int p = 0; p < PF; ++p)
#pragma unroll
      for (int j = 0; j < TN; ++j) acc[j] = mfma16(a[p], b[p][j], acc[j]);
  }
  __builtin_amdgcn_sched_barrier(0);
  asm volatile("s_nop 15");
  __builtin_amdgcn_sched_barrier(0);
#pragma unroll
  for (int j = 0; j < TN; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) part[w][4 * q + i][16 * j + r] = acc[j][i];
  __syncthreads();
  for (int i = threadIdx.x; i < NR_ROWS * 16 * TN; i += 64 * NW) {
    const int row = i / (16 * TN), n = i - row * 16 * TN;
    float z = 0.f;
#pragma unroll
    for (int k = 0; k < NW; ++k) z += part[k][row][n];
    part[0][row][n] = z;
  }
  __syncthreads();
}

template <int TN>
__global__ __launch_bounds__(64 * nr_waves(TN)) void narrow_linear_kernel(const bf16* __restrict__ x, int64_t xs,
                                                            const bf16* __restrict__ wt, const float* __restrict__ bias,
                                                            int N, int K, float* __restrict__ out, int64_t os,
                                                            int64_t T) {
  __shared__ float part[nr_waves(TN)][NR_ROWS][nr_ld(TN)];
  narrow_product<TN>(x, xs, T, wt, N, K, part);
  for (int i = threadIdx.x; i < NR_ROWS * N; i += 64 * nr_waves(TN)) {
    const int row = i / N, n = i - row * N;
    const int64_t t = (int64_t)blockIdx.x * NR_ROWS + row;
    if (t < T) out[t * os + n] = part[0][row][n] + (bias != nullptr ? bias[n] : 0.f);
  }
}

// softmax over all N experts, the k largest (ties: the lower index), their scores as weights (norm: divided by their sum)
// times scale; lane = expert
template <int TN>
__global__ __launch_bounds__(64 * nr_waves(TN)) void narrow_route_kernel(const bf16* __restrict__ x, int64_t xs,
                                                           const bf16* __restrict__ wt, int N, int K, int k, bool norm,
                                                           float scale, float* __restrict__ tw, int* __restrict__ te,
                                                           int64_t T) {
  __shared__ float part[nr_waves(TN)][NR_ROWS][nr_ld(TN)];
  narrow_product<TN>(x, xs, T, wt, N, K, part);
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
#pragma unroll 1
  for (int row = w; row < NR_ROWS; row += nr_waves(TN)) {
    const int64_t t = (int64_t)blockIdx.x * NR_ROWS + row;
    if (t >= T) break;   // (uniform)
    const float z = lane < N ? part[0][row][lane] : -INFINITY;
    const float mx = wave_max(z), ex = lane < N ? expf(z - mx) : 0.f;
    const float s = ex / wave_sum(ex);
    float c = lane < N ? s : -1.f, mine = 0.f, sum = 0.f;
    int me = 0;
    for (int j = 0; j < k; ++j) {
      float bv = c;
      int bi = lane;
#pragma unroll
      for (int o = 32; o > 0; o >>= 1) {
        const float ov = __shfl_xor(bv, o, 64);
        const int oi = __shfl_xor(bi, o, 64);
        if (ov > bv || (ov == bv && oi < bi)) {
          bv = ov;
          bi = oi;
        }
      }
      if (lane == j) {
        mine = bv;
        me = bi;
      }
      if (lane == bi) c = -1.f;
      sum += bv;
    }
    if (lane < k) {
      tw[t * k + lane] = (norm ? mine / sum : mine) * scale;
      te[t * k + lane] = me;
    }
  }
}

}  // namespace mw
}  // namespace kafka

using namespace kafka;
using namespace kafka::mw;

extern "C" {

int kafka_moe_sort_max_e() { return SORT_MAXE; }

hipError_t kafka_launch_moe_sort(const float* topk_w, const int* topk_e, int n, int k, int E, int bm, int* perm_tok,
                                 float* perm_w, int* expert_off, int* tile_off, int* inv, hipStream_t st) {
  if (n < 1) return hipSuccess;
  if (E < 1 || E > SORT_MAXE || k < 1 || bm < 1) return hipErrorInvalidValue;
  int bits = 0;
  while ((1 << bits) < E) ++bits;
  moe_sort_kernel<<<1, SORT_NT, 0, st>>>(topk_w, topk_e, n, k, E, bits, bm, perm_tok, perm_w, expert_off, tile_off,
                                        inv);
  return hipGetLastError();
}

// epi: 0 gate_up -> silu(gate) * up (or clamped) into Y [n_ent][N / 2], 1 relu squared into Y [n_ent][N], 2 combine into
// out [T][N], 3 weighted rows into Y [n_ent][N]
hipError_t kafka_launch_grouped_wide(const bf16* X, int64_t ldx, const bf16* Wt, int E, int N, int K,
                                     const int* perm_tok, const float* perm_w, const int* expert_off, int n_ent,
                                     int gather, int epi, bf16* Y, int64_t ldy, float* out, int64_t ldo,
                                     float glu_limit, float glu_alpha, hipStream_t st) {
  if (n_ent < 1 || E < 1) return hipSuccess;
  if (N % 64 || K % (2 * BK) || N < 64 || K < 2 * BK || epi < 0 || epi > 3 || (epi == EPI_COMBINE) != (out != nullptr) ||
      (epi != EPI_COMBINE) != (Y != nullptr))
    return hipErrorInvalidValue;
  const int64_t items = ((int64_t)n_ent / BM + E) * ((N + BN - 1) / BN);   // an upper bound over all routings
  if (items > 0x0fffffff) return hipErrorInvalidValue;
  const unsigned grid = (unsigned)((items + 7) / 8 * 8);
  const auto* wt = reinterpret_cast<const bf16x8*>(Wt);
  auto a = [&](auto kern) {
    kern<<<grid, 256, 0, st>>>(X, ldx, wt, E, N, K, perm_tok, perm_w, expert_off, Y, ldy, out, ldo, glu_limit, glu_alpha);
  };
  if (gather) {
    if (epi == EPI_GLU) a(grouped_wide_kernel<true, EPI_GLU>);
    else if (epi == EPI_RELU2) a(grouped_wide_kernel<true, EPI_RELU2>);
    else if (epi == EPI_ROWS) a(grouped_wide_kernel<true, EPI_ROWS>);
    else a(grouped_wide_kernel<true, EPI_COMBINE>);
  } else {
    if (epi == EPI_GLU) a(grouped_wide_kernel<false, EPI_GLU>);
    else if (epi == EPI_RELU2) a(grouped_wide_kernel<false, EPI_RELU2>);
    else if (epi == EPI_ROWS) a(grouped_wide_kernel<false, EPI_ROWS>);
    else a(grouped_wide_kernel<false, EPI_COMBINE>);
  }
  return hipGetLastError();
}

// bf16 rows and weights in 16-byte pieces, up to 64 weight rows
int kafka_narrow_ok(int N, int K, int64_t xs) { return N >= 1 && N <= NR_MAXN && K >= 32 && K % 32 == 0 && xs % 8 == 0; }
int kafka_narrow_max_k() { return NR_MAXK; }

hipError_t kafka_launch_narrow_linear(const bf16* x, int64_t xs, const bf16* w, const float* bias, int N, int K,
                                      float* out, int64_t os, int64_t T, hipStream_t st) {
  if (T <= 0) return hipSuccess;
  if (!kafka_narrow_ok(N, K, xs)) return hipErrorInvalidValue;
  const unsigned g = (unsigned)((T + NR_ROWS - 1) / NR_ROWS);
  auto a = [&](auto kern, int tn) { kern<<<g, 64 * nr_waves(tn), 0, st>>>(x, xs, w, bias, N, K, out, os, T); };
  if (N <= 16) a(narrow_linear_kernel<1>, 1);
  else if (N <= 32) a(narrow_linear_kernel<2>, 2);
  else if (N <= 48) a(narrow_linear_kernel<3>, 3);
  else a(narrow_linear_kernel<4>, 4);
  return hipGetLastError();
}

hipError_t kafka_launch_narrow_route(const bf16* x, int64_t xs, const bf16* w, int N, int K, int k, int norm, float scale,
                                     float* tw, int* te, int64_t T, hipStream_t st) {
  if (T <= 0) return hipSuccess;
  if (!kafka_narrow_ok(N, K, xs) || k < 1 || k > N || k > NR_MAXK) return hipErrorInvalidValue;
  const unsigned g = (unsigned)((T + NR_ROWS - 1) / NR_ROWS);
  auto a = [&](auto kern, int tn) {
    kern<<<g, 64 * nr_waves(tn), 0, st>>>(x, xs, w, N, K, k, norm != 0, scale, tw, te, T);
  };
  if (N <= 16) a(narrow_route_kernel<1>, 1);
  else if (N <= 32) a(narrow_route_kernel<2>, 2);
  else if (N <= 48) a(narrow_route_kernel<3>, 3);
  else a(narrow_route_kernel<4>, 4);
  return hipGetLastError();
}

}  // extern "C"
