// K7 SiLU-and-mul: out[t, i] = silu(x[t, i]) * x[t, I + i] over the fused gate_up
// projection output.  16-byte vector loads/stores (8 halves per lane), one vector
// per thread on a 2-D grid (memory-bound; no index division).
#include <algorithm>

#include "common.h"
#include "launch.h"

namespace kgc {

// grid (ceil(I/8/256), rows): one 16-byte vector per thread, no index division.  Rows of x and
// out may be column slices of wider matrices (strides xs, os).
template <typename T>
__global__ __launch_bounds__(256) void silu_mul_kernel(T* __restrict__ out, int64_t os,
                                                       const T* __restrict__ x, int64_t xs, int I) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c * 8 >= I) return;
  const int64_t r = blockIdx.y;
  const T* xr = x + r * xs;
  Pack8<T> g, u, o;
  g.u = *reinterpret_cast<const u32x4*>(xr + c * 8);
  u.u = *reinterpret_cast<const u32x4*>(xr + I + c * 8);
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const float gf = to_f(g.h[j]);
    o.h[j] = from_f<T>(gf / (1.f + __expf(-gf)) * to_f(u.h[j]));
  }
  *reinterpret_cast<u32x4*>(out + r * os + c * 8) = o.u;
}

// any element type, any I and any alignment
template <typename T>
__global__ __launch_bounds__(256) void silu_mul_any_kernel(T* __restrict__ out, int64_t os,
                                                           const T* __restrict__ x, int64_t xs,
                                                           int I) {
  const int64_t r = blockIdx.y;
  const T* xr = x + r * xs;
  for (int c = blockIdx.x * 256 + threadIdx.x; c < I; c += gridDim.x * 256) {
    const float gf = to_f(xr[c]);
    out[r * os + c] = from_f<T>(gf / (1.f + expf(-gf)) * to_f(xr[I + c]));
  }
}

template <typename T>
static void silu_mul_rows(T* out, int64_t os, const T* x, int64_t xs, int64_t rows, int I,
                          hipStream_t s) {
  bool vec = !std::is_same_v<T, float> && I % 8 == 0 && xs % 8 == 0 && os % 8 == 0 &&
             reinterpret_cast<uintptr_t>(x) % 16 == 0 && reinterpret_cast<uintptr_t>(out) % 16 == 0;
  for (int64_t r0 = 0; r0 < rows; r0 += 65535) {   // gridDim.y <= 65535
    const unsigned n = (unsigned)std::min<int64_t>(rows - r0, 65535);
    if constexpr (!std::is_same_v<T, float>) {
      if (vec) {
        silu_mul_kernel<T><<<dim3(((I >> 3) + 255) / 256, n), 256, 0, s>>>(
            out + r0 * os, os, x + r0 * xs, xs, I);
        continue;
      }
    }
    silu_mul_any_kernel<T><<<dim3(std::min((I + 255) / 256, 64), n), 256, 0, s>>>(
        out + r0 * os, os, x + r0 * xs, xs, I);
  }
}

void launch_silu_mul(int dtype, void* out, int64_t os, const void* x, int64_t xs, int64_t rows,
                     int I, hipStream_t s) {
  if (dtype == DT_F32) silu_mul_rows<float>((float*)out, os, (const float*)x, xs, rows, I, s);
  else if (dtype == DT_BF16) silu_mul_rows<bf16>((bf16*)out, os, (const bf16*)x, xs, rows, I, s);
  else silu_mul_rows<f16>((f16*)out, os, (const f16*)x, xs, rows, I, s);
}

// ---- tanh cap on the logits -----------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void logit_softcap_kernel(float* __restrict__ out,
                                                            const T* __restrict__ x, int64_t xs,
                                                            int V, float cap, float inv) {
  const int64_t r = blockIdx.y;
  for (int c = blockIdx.x * 256 + threadIdx.x; c < V; c += gridDim.x * 256)
    out[r * V + c] = cap * tanhf(to_f(x[r * xs + c]) * inv);
}

void launch_logit_softcap(int dtype, float* out, const void* x, int64_t xs, int64_t rows, int V,
                          float cap, hipStream_t s) {
  for (int64_t r0 = 0; r0 < rows; r0 += 65535) {
    const dim3 grid(std::min((V + 255) / 256, 128), (unsigned)std::min<int64_t>(rows - r0, 65535));
    float* o = out + r0 * V;
    if (dtype == DT_BF16)
      logit_softcap_kernel<bf16><<<grid, 256, 0, s>>>(o, (const bf16*)x + r0 * xs, xs, V, cap, 1.f / cap);
    else if (dtype == DT_F16)
      logit_softcap_kernel<f16><<<grid, 256, 0, s>>>(o, (const f16*)x + r0 * xs, xs, V, cap, 1.f / cap);
    else
      logit_softcap_kernel<float><<<grid, 256, 0, s>>>(o, (const float*)x + r0 * xs, xs, V, cap, 1.f / cap);
  }
}

// ---- PolyNorm, clamped gated activation, scaled embedding + learned positions --------------
namespace {

#define KGC_ACT_DISPATCH_T(dtype, ...)                      \
  do {                                                      \
    if ((dtype) == DT_BF16) { typedef bf16 T; __VA_ARGS__; } \
    else if ((dtype) == DT_F16) { typedef f16 T; __VA_ARGS__; } \
    else { typedef float T; __VA_ARGS__; }                  \
  } while (0)

// VEC consecutive elements of a row as fp32 (one 16-byte load of 8 halves when VEC = 8)
template <typename T, int VEC>
__device__ __forceinline__ void load_row(const T* p, float (&v)[VEC]) {
  if constexpr (VEC == 8 && !std::is_same_v<T, float>) {
    Pack8<T> t;
    t.u = *reinterpret_cast<const u32x4*>(p);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = to_f(t.h[e]);
  } else {
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = to_f(p[e]);
  }
}

template <typename T, int VEC>
__device__ __forceinline__ void store_row(T* p, const float (&v)[VEC]) {
  if constexpr (VEC == 8 && !std::is_same_v<T, float>) {
    Pack8<T> t;
#pragma unroll
    for (int e = 0; e < 8; ++e) t.h[e] = from_f<T>(v[e]);
    *reinterpret_cast<u32x4*>(p) = t.u;
  } else {
#pragma unroll
    for (int e = 0; e < VEC; ++e) p[e] = from_f<T>(v[e]);
  }
}

// out = a z / rms(z) + b z^2 / rms(z^2) + c z^3 / rms(z^3) + e per row, rms(v) =
// sqrt(mean(v^2) + eps); one workgroup per row, two passes (the second one reads the row
// from cache), fp32 sums.  VEC = 8: 16-bit rows whose length is a multiple of 8.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void polynorm_kernel(T* __restrict__ out,
                                                       const T* __restrict__ z,
                                                       const float* __restrict__ coef, int F,
                                                       float eps) {
  __shared__ float scratch[4];
  const int64_t row = blockIdx.x;
  const T* zr = z + row * F;
  T* orow = out + row * F;
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  for (int c = threadIdx.x * VEC; c < F; c += 256 * VEC) {
    float v[VEC];
    load_row<T, VEC>(zr + c, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float q = v[e] * v[e];
      s2 += q;
      s4 += q * q;
      s6 += q * q * q;
    }
  }
  s2 = block_sum<256>(s2, scratch);
  s4 = block_sum<256>(s4, scratch);
  s6 = block_sum<256>(s6, scratch);
  const float n = (float)F;
  const float a = coef[0] / sqrtf(s2 / n + eps), b = coef[1] / sqrtf(s4 / n + eps),
              cc = coef[2] / sqrtf(s6 / n + eps), e0 = coef[3];
  for (int c = threadIdx.x * VEC; c < F; c += 256 * VEC) {
    float v[VEC];
    load_row<T, VEC>(zr + c, v);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float x = v[e];
      v[e] = ((cc * x + b) * x + a) * x + e0;
    }
    store_row<T, VEC>(orow + c, v);
  }
}

// x [rows, 2 I] = gate | up  ->  g sigmoid(alpha g) (u + 1), g = min(gate, limit),
// u = clamp(up, -limit, limit)
template <typename T, int VEC>
__global__ __launch_bounds__(256) void swiglu_clamp_kernel(T* __restrict__ out,
                                                           const T* __restrict__ x,
                                                           int64_t rows, int I, float limit,
                                                           float alpha) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (c >= I) return;
  for (int64_t r = blockIdx.y; r < rows; r += gridDim.y) {
    const T* xr = x + r * 2 * I;
    float g[VEC], u[VEC];
    load_row<T, VEC>(xr + c, g);
    load_row<T, VEC>(xr + I + c, u);
#pragma unroll
    for (int e = 0; e < VEC; ++e) {
      const float gv = fminf(g[e], limit), uv = fminf(fmaxf(u[e], -limit), limit);
      g[e] = gv / (1.f + expf(-alpha * gv)) * (uv + 1.f);
    }
    store_row<T, VEC>(out + r * I + c, g);
  }
}

// A gated pair of a scaled input: silu(w g) * (w u)
__device__ __forceinline__ float scaled_silu(float g, float u, float w) {
  const float gv = w * g;
  return gv / (1.f + expf(-gv)) * (w * u);
}

// Every expert's activation for every token: x [T, E 2 I + 2 Is] = per expert gate | up, then the
// shared expert's -> out [T, E I + Is]; w [T, k] / ids [T, k]: the token's experts and their
// weights, zeros for the others, 1 for the shared one.  VEC adjacent columns lie in one expert.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void expert_silu_all_kernel(
    T* __restrict__ out, const T* __restrict__ x, const float* __restrict__ w,
    const int* __restrict__ ids, int E, int k, int I, int Is) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC, n = E * I + Is;
  if (c >= n) return;
  const int64_t t = blockIdx.y;
  const int e = c < E * I ? c / I : E, i = c - e * I, len = e < E ? I : Is;
  float we = e < E ? 0.f : 1.f;
  for (int j = 0; j < k; ++j)
    if (ids[t * k + j] == e) we = w[t * k + j];
  float o[VEC];
  if (we == 0.f) {
#pragma unroll
    for (int q = 0; q < VEC; ++q) o[q] = 0.f;
  } else {
    const T* xr = x + t * 2 * n + (int64_t)e * 2 * I + i;
    float g[VEC], u[VEC];
    load_row<T, VEC>(xr, g);
    load_row<T, VEC>(xr + len, u);
#pragma unroll
    for (int q = 0; q < VEC; ++q) o[q] = scaled_silu(g[q], u[q], we);
  }
  store_row<T, VEC>(out + t * n + c, o);
}

// Expert-sorted rows: out [rows, I] from x [rows, 2 I] = gate | up, row r scaled by the weight of
// its pair sorted_ids[r]; rows without a pair (>= npairs) are left as they are.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void expert_silu_rows_kernel(
    T* __restrict__ out, const T* __restrict__ x, const float* __restrict__ w,
    const int* __restrict__ sorted_ids, int npairs, int64_t rows, int I) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (c >= I) return;
  for (int64_t r = blockIdx.y; r < rows; r += gridDim.y) {
    const int p = sorted_ids[r];
    if (p < 0 || p >= npairs) continue;
    const float we = w[p];
    float g[VEC], u[VEC];
    load_row<T, VEC>(x + r * 2 * I + c, g);
    load_row<T, VEC>(x + r * 2 * I + I + c, u);
#pragma unroll
    for (int q = 0; q < VEC; ++q) g[q] = scaled_silu(g[q], u[q], we);
    store_row<T, VEC>(out + r * I + c, g);
  }
}

// out fp32 [T, W] = table[ids[t]] * scale + pos[positions[t]]
template <typename T>
__global__ __launch_bounds__(256) void embed_pos_kernel(
    float* __restrict__ out, const int64_t* __restrict__ ids,
    const int64_t* __restrict__ positions, const T* __restrict__ table,
    const float* __restrict__ pos, int W, int vocab, int max_pos, float scale) {
  const int64_t t = blockIdx.x;
  int64_t id = ids[t], p = positions[t];
  if (id < 0 || id >= vocab) id = 0;                  // padding rows carry any id
  if (p < 0) p = 0;
  if (p >= max_pos) p = max_pos - 1;
  const T* er = table + id * W;
  const float* pr = pos != nullptr ? pos + p * W : nullptr;
  for (int c = threadIdx.x; c < W; c += 256) {
    float v = to_f(er[c]) * scale;
    if (pr != nullptr) v += pr[c];
    out[t * W + c] = v;
  }
}

}  // namespace

void launch_polynorm(int dtype, void* out, const void* z, const float* coef, int64_t rows, int F,
                     float eps, hipStream_t s) {
  if (rows <= 0 || F <= 0) return;
  const bool vec = dtype != DT_F32 && F % 8 == 0 && reinterpret_cast<uintptr_t>(z) % 16 == 0 &&
                   reinterpret_cast<uintptr_t>(out) % 16 == 0;
  if (vec)
    KGC_ACT_DISPATCH_T(dtype, polynorm_kernel<T, 8><<<rows, 256, 0, s>>>(
        (T*)out, (const T*)z, coef, F, eps));
  else
    KGC_ACT_DISPATCH_T(dtype, polynorm_kernel<T, 1><<<rows, 256, 0, s>>>(
        (T*)out, (const T*)z, coef, F, eps));
}

void launch_swiglu_clamp(int dtype, void* out, const void* x, int64_t rows, int I, float limit,
                         float alpha, hipStream_t s) {
  if (rows <= 0 || I <= 0) return;
  const bool vec = dtype != DT_F32 && I % 8 == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0 &&
                   reinterpret_cast<uintptr_t>(out) % 16 == 0;
  const int per = 256 * (vec ? 8 : 1);
  const dim3 grid((I + per - 1) / per, (unsigned)(rows < 65535 ? rows : 65535));
  if (vec)
    KGC_ACT_DISPATCH_T(dtype, swiglu_clamp_kernel<T, 8><<<grid, 256, 0, s>>>(
        (T*)out, (const T*)x, rows, I, limit, alpha));
  else
    KGC_ACT_DISPATCH_T(dtype, swiglu_clamp_kernel<T, 1><<<grid, 256, 0, s>>>(
        (T*)out, (const T*)x, rows, I, limit, alpha));
}

void launch_expert_silu_all(int dtype, void* out, const void* x, const float* w, const int* ids,
                            int T_, int E, int k, int I, int Is, hipStream_t s) {
  const int n = E * I + Is;
  if (T_ <= 0 || n <= 0) return;
  const bool vec = dtype != DT_F32 && I % 8 == 0 && Is % 8 == 0 &&
                   reinterpret_cast<uintptr_t>(x) % 16 == 0 && reinterpret_cast<uintptr_t>(out) % 16 == 0;
  const int per = 256 * (vec ? 8 : 1);
  for (int t0 = 0; t0 < T_; t0 += 65535) {         // gridDim.y <= 65535
    const dim3 grid((n + per - 1) / per, std::min(T_ - t0, 65535));
    const float* wt = w + (int64_t)t0 * k;
    const int* it = ids + (int64_t)t0 * k;
#define KGC_ESA(V)                                                                             \
  KGC_ACT_DISPATCH_T(dtype, expert_silu_all_kernel<T, V><<<grid, 256, 0, s>>>(                 \
      (T*)out + (int64_t)t0 * n, (const T*)x + (int64_t)t0 * 2 * n, wt, it, E, k, I, Is))
    if (vec) KGC_ESA(8); else KGC_ESA(1);
#undef KGC_ESA
  }
}

void launch_expert_silu_rows(int dtype, void* out, const void* x, const float* w,
                             const int* sorted_ids, int npairs, int64_t rows, int I,
                             hipStream_t s) {
  if (rows <= 0 || I <= 0) return;
  const bool vec = dtype != DT_F32 && I % 8 == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0 &&
                   reinterpret_cast<uintptr_t>(out) % 16 == 0;
  const int per = 256 * (vec ? 8 : 1);
  const dim3 grid((I + per - 1) / per, (unsigned)std::min<int64_t>(rows, 65535));
  if (vec)
    KGC_ACT_DISPATCH_T(dtype, expert_silu_rows_kernel<T, 8><<<grid, 256, 0, s>>>(
        (T*)out, (const T*)x, w, sorted_ids, npairs, rows, I));
  else
    KGC_ACT_DISPATCH_T(dtype, expert_silu_rows_kernel<T, 1><<<grid, 256, 0, s>>>(
        (T*)out, (const T*)x, w, sorted_ids, npairs, rows, I));
}

void launch_embed_pos(int dtype, float* out, const int64_t* ids, const int64_t* positions,
                      const void* table, const float* pos, int T_, int W, int vocab, int max_pos,
                      float scale, hipStream_t s) {
  if (T_ <= 0) return;
  KGC_ACT_DISPATCH_T(dtype, embed_pos_kernel<T><<<T_, 256, 0, s>>>(
      out, ids, positions, (const T*)table, pos, W, vocab, max_pos, scale));
}

}  // namespace kgc
