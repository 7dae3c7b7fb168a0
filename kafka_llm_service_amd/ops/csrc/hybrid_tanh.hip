// Kernels of residual streams with element-wise tanh norms, for gfx950.
//
//   add_tanh_norm   x += y1 + y2 (or x = y1 + y2) on the fp32 stream and, from the new x, up to two outputs
//                   tanh(alpha x) * w + b and a copy, in the activation dtype. y1 may be the split-K slabs of a projection
//                   (summed while loading), y2 a token's routed expert rows (gathered while loading); every part is
//                   optional.
//
// Built for bf16 and fp32 activations; the stream, the sums and the norms are fp32 in both. Sizes are run-time values
// with no alignment assumptions (four columns per thread where sizes and strides allow).
#include "common.h"

namespace kafka {
namespace ht {

template <typename T>
__device__ __forceinline__ float ldf(const T* p) { return (float)(*p); }
template <typename T>
__device__ __forceinline__ void stf(T* p, float v) { *p = (T)v; }

constexpr int NT = 256;
constexpr int TN_MAXS = 8;   // split-K slabs of y1

// tanh: near zero its Taylor polynomial (relative error below 1e-7 up to 0.3), else 1 - 2 / (1 + e^(2|z|)); e^(2|z|)
// overflows to infinity for large |z|, which gives 1
__device__ __forceinline__ float tanh_f(float z) {
  const float a = fabsf(z), z2 = z * z;
  const float p = z * (1.f + z2 * (-1.f / 3.f + z2 * (2.f / 15.f + z2 * (-17.f / 315.f + z2 * (62.f / 2835.f)))));
  const float e = fast_exp2(a * 2.8853900817779268f);
  const float q = copysignf(1.f - 2.f * __builtin_amdgcn_rcpf(1.f + e), z);
  return a < 0.3f ? p : q;
}

struct TanhNorms {
  int n;                  // norms (0 .. 2)
  float alpha[2];
  const float* w[2];
  const float* b[2];
  void* out[2];
  int64_t os[2];
};

// grid (column blocks of NT * VEC, row blocks of `rows`); S: slabs of an fp32 y1, 0 = y1 in the activation dtype
template <typename AT, int VEC, int S>
__global__ __launch_bounds__(NT) void add_tanh_norm_kernel(float* __restrict__ x, int64_t xs,
                                                           const void* __restrict__ y1, int64_t y1s, int64_t slab,
                                                           const float* __restrict__ y2, int64_t y2s,
                                                           const AT* __restrict__ er, int64_t ers,
                                                           const int* __restrict__ inv, int ek, bool assign,
                                                           TanhNorms nm, AT* __restrict__ copy, int64_t cs, int64_t T,
                                                           int d, int rows) {
  const int i = ((int)blockIdx.x * NT + (int)threadIdx.x) * VEC;
  if (i >= d) return;
  float w[2][VEC], b[2][VEC];
#pragma unroll
  for (int k = 0; k < 2; ++k)
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      w[k][e] = k < nm.n ? nm.w[k][i + e] : 0.f;
      b[k][e] = k < nm.n ? nm.b[k][i + e] : 0.f;
    }
  const int64_t t1 = min(T, (int64_t)(blockIdx.y + 1) * rows);
  for (int64_t t = (int64_t)blockIdx.y * rows; t < t1; ++t) {
    float v[VEC];
    float* xr = x + t * xs + i;
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = assign ? 0.f : xr[e];
    if (y1 != nullptr) {
      float y[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) y[e] = 0.f;
      if constexpr (S > 0) {
        const float* p = reinterpret_cast<const float*>(y1) + t * y1s + i;
#pragma unroll
        for (int s = 0; s < S; ++s)
#pragma unroll
          for (int e = 0; e < VEC; ++e) y[e] += p[s * slab + e];
      } else {
        const AT* p = reinterpret_cast<const AT*>(y1) + t * y1s + i;
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[e] = ldf(p + e);
      }
      if (y2 != nullptr) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[e] += y2[t * y2s + i + e];
      }
      if (er != nullptr) {   // in the order of the token's choices
        constexpr int PF = 4;
        for (int j0 = 0; j0 < ek; j0 += PF) {
          AT z[PF][VEC];
#pragma unroll
          for (int j = 0; j < PF; ++j) {
            const AT* p = er + (int64_t)inv[t * ek + min(j0 + j, ek - 1)] * ers + i;
#pragma unroll
            for (int e = 0; e < VEC; ++e) z[j][e] = p[e];
          }
#pragma unroll
          for (int j = 0; j < PF; ++j)
            if (j0 + j < ek)
#pragma unroll
              for (int e = 0; e < VEC; ++e) y[e] += (float)z[j][e];
        }
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) v[e] += y[e];
#pragma unroll
      for (int e = 0; e < VEC; ++e) xr[e] = v[e];
    }
    if (copy != nullptr) {
#pragma unroll
      for (int e = 0; e < VEC; ++e) stf(copy + t * cs + i + e, v[e]);
    }
#pragma unroll
    for (int k = 0; k < 2; ++k)
      if (k < nm.n) {
        AT* o = reinterpret_cast<AT*>(nm.out[k]) + t * nm.os[k] + i;
#pragma unroll
        for (int e = 0; e < VEC; ++e) stf(o + e, tanh_f(nm.alpha[k] * v[e]) * w[k][e] + b[k][e]);
      }
  }
}

}  // namespace ht
}  // namespace kafka

using namespace kafka::ht;

extern "C" {

int kafka_hy_add_tanh_norm_max_slabs() { return TN_MAXS; }

// y1_f32: y1 is fp32 with S slabs (S >= 1), else of the activation dtype
hipError_t kafka_hy_add_tanh_norm(int f32, float* x, int64_t xs, const void* y1, int64_t y1s, int y1_f32, int S,
                                  int64_t slab, const float* y2, int64_t y2s, const void* er, int64_t ers,
                                  const int* inv, int ek, int assign, int n_norms, const float* alpha,
                                  const float* const* w, const float* const* b, void* const* out, const int64_t* os,
                                  void* copy, int64_t cs, int64_t T, int d, hipStream_t st) {
  if (T <= 0 || d <= 0) return hipSuccess;
  if (n_norms < 0 || n_norms > 2 || S < 1 || S > TN_MAXS) return hipErrorInvalidValue;
  TanhNorms nm{};
  nm.n = n_norms;
  // four columns a thread: 16-byte pieces of fp32 rows, 8-byte ones of bf16 rows
  auto al = [](const void* p, int64_t stride, size_t bytes) {
    return p == nullptr || ((reinterpret_cast<uintptr_t>(p) & (bytes - 1)) == 0 && stride % 4 == 0);
  };
  const size_t ab = f32 ? 16 : 8;
  bool v4 = d % 4 == 0 && al(x, xs, 16) && al(y1, y1s, y1_f32 ? 16 : ab) && slab % 4 == 0 && al(y2, y2s, 16) &&
            al(copy, cs, ab) && al(er, ers, ab);
  for (int k = 0; k < n_norms; ++k) {
    nm.alpha[k] = alpha[k]; nm.w[k] = w[k]; nm.b[k] = b[k]; nm.out[k] = out[k]; nm.os[k] = os[k];
    v4 = v4 && al(w[k], 0, 16) && al(b[k], 0, 16) && al(out[k], os[k], ab);
  }
  const int per = NT * (v4 ? 4 : 1), gx = (d + per - 1) / per;
  int rows = 1;   // rows that share the norms' weights in registers, as long as the launch fills the chip
  while (rows < 8 && (T / (2 * rows)) * gx >= 2048) rows *= 2;
  while ((T + rows - 1) / rows > 65535) rows *= 2;
  const dim3 grid(gx, (unsigned)((T + rows - 1) / rows));
  auto a = [&](auto k, auto* tag) {
    using AT = std::remove_pointer_t<decltype(tag)>;
    k<<<grid, NT, 0, st>>>(x, xs, y1, y1s, slab, y2, y2s, (const AT*)er, ers, inv, ek, assign != 0, nm, (AT*)copy, cs, T, d, rows);
  };
#define TN_S(AT, V)                                                                 \
  do {                                                                              \
    AT* tag = nullptr;                                                              \
    switch (y1_f32 ? S : 0) {                                                       \
      case 0: a(add_tanh_norm_kernel<AT, V, 0>, tag); break;                        \
      case 1: a(add_tanh_norm_kernel<AT, V, 1>, tag); break;                        \
      case 2: a(add_tanh_norm_kernel<AT, V, 2>, tag); break;                        \
      case 3: a(add_tanh_norm_kernel<AT, V, 3>, tag); break;                        \
      case 4: a(add_tanh_norm_kernel<AT, V, 4>, tag); break;                        \
      case 5: a(add_tanh_norm_kernel<AT, V, 5>, tag); break;                        \
      case 6: a(add_tanh_norm_kernel<AT, V, 6>, tag); break;                        \
      case 7: a(add_tanh_norm_kernel<AT, V, 7>, tag); break;                        \
      default: a(add_tanh_norm_kernel<AT, V, 8>, tag); break;                       \
    }                                                                               \
  } while (0)
  if (f32) {
    if (v4) TN_S(float, 4); else TN_S(float, 1);
  } else {
    if (v4) TN_S(bf16, 4); else TN_S(bf16, 1);
  }
#undef TN_S
  return hipGetLastError();
}

}  // extern "C"
