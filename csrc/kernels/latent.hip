// Kernels of latent attention with latent queries:
//   latent_down_store  one merged projection row -> normed query latent, cache row [normed
//                      key/value latent | rotated key part], sigmoid of the head gates
//   head_gemm          one small matrix per head (queries into latent space, attention results
//                      out of it), with the rotation of the queries' rotary part in the same launch
#include <algorithm>

#include "common.h"
#include "launch.h"

namespace kgc {

#define KGC_DISPATCH_T(dtype, ...)                          \
  do {                                                      \
    if ((dtype) == DT_BF16) { typedef bf16 T; __VA_ARGS__; } \
    else if ((dtype) == DT_F16) { typedef f16 T; __VA_ARGS__; } \
    else { typedef float T; __VA_ARGS__; }                  \
  } while (0)

namespace {

// One workgroup per token.  row = [qr | rank | r | gates ...]; both latents over their root mean
// squares times a weight, the rotary key part turned by the position (pairs (2i, 2i + 1), table
// row cos[r/2] | sin[r/2]).  fp32 sums, one barrier.
template <typename T>
__global__ __launch_bounds__(256) void latent_down_store_kernel(
    T* __restrict__ cq, float* __restrict__ gate, const T* __restrict__ proj, int64_t ps,
    const int64_t* __restrict__ positions, const float* __restrict__ table, int table_rows,
    const float* __restrict__ qw, const float* __restrict__ kw, float eps, T* __restrict__ cache,
    const int64_t* __restrict__ slots, int64_t cache_rows, int qr, int rank, int r, int gates) {
  __shared__ float scratch[2][4];
  const int64_t t = blockIdx.x;
  const T* row = proj + t * ps;
  const T* kv = row + qr;
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x; c < qr; c += 256) {
    const float v = to_f(row[c]);
    sq += v * v;
  }
  for (int c = threadIdx.x; c < rank; c += 256) {
    const float v = to_f(kv[c]);
    sk += v * v;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((threadIdx.x & 63) == 0) {
    scratch[0][threadIdx.x >> 6] = sq;
    scratch[1][threadIdx.x >> 6] = sk;
  }
  __syncthreads();
  sq = (scratch[0][0] + scratch[0][1]) + (scratch[0][2] + scratch[0][3]);
  sk = (scratch[1][0] + scratch[1][1]) + (scratch[1][2] + scratch[1][3]);
  const float rq = 1.f / sqrtf(sq / (float)qr + eps), rk = 1.f / sqrtf(sk / (float)rank + eps);
  for (int c = threadIdx.x; c < qr; c += 256) cq[t * qr + c] = from_f<T>(to_f(row[c]) * rq * qw[c]);
  for (int c = threadIdx.x; c < gates; c += 256)
    gate[t * gates + c] = 1.f / (1.f + expf(-to_f(kv[rank + r + c])));
  const int64_t slot = slots[t];
  if (slot < 0 || slot >= cache_rows) return;
  T* crow = cache + slot * (rank + r);
  for (int c = threadIdx.x; c < rank; c += 256) crow[c] = from_f<T>(to_f(kv[c]) * rk * kw[c]);
  if (r > 0) {
    int64_t pos = positions[t];
    if (pos < 0) pos = 0;
    if (pos >= table_rows) pos = table_rows - 1;      // host checks max_pos; never read past
    const float* cs = table + pos * r;
    for (int p = threadIdx.x; p < (r >> 1); p += 256) {
      float oa, ob;
      neox_rot(to_f(kv[rank + 2 * p]), to_f(kv[rank + 2 * p + 1]), cs[p], cs[(r >> 1) + p], oa, ob);
      crow[rank + 2 * p] = from_f<T>(oa);
      crow[rank + 2 * p + 1] = from_f<T>(ob);
    }
  }
}

// the rotary columns of the output: thread e takes pair e % (r/2) of token e / (r/2), head h
template <typename T>
__device__ __forceinline__ void rotate_rows(const HeadGemm& a, int h, int first, int step) {
  const T* rot = static_cast<const T*>(a.rot);
  T* out = static_cast<T*>(a.out);
  const int half = a.r >> 1, n = a.T * half;
  for (int e = first; e < n; e += step) {
    const int t = e / half, p = e - t * half;
    int64_t pos = a.positions[t];
    if (pos < 0) pos = 0;
    if (pos >= a.table_rows) pos = a.table_rows - 1;
    const float* cs = a.table + pos * a.r;
    const T* src = rot + t * a.rs + h * a.rh + 2 * p;
    T* dst = out + t * a.os + h * a.oh + a.N + 2 * p;
    float oa, ob;
    neox_rot(to_f(src[0]), to_f(src[1]), cs[p], cs[half + p], oa, ob);
    dst[0] = from_f<T>(oa);
    dst[1] = from_f<T>(ob);
  }
}

// Matrix cores (16-bit types, K % 8 == 0, K <= 32 KS, N % 4 == 0, 16-byte rows).  A workgroup owns
// 64 outputs of one head: their weights stay in registers as A fragments (row = output) while
// its four waves walk the tokens 16 at a time (B fragments: column = token, straight from the
// rows), so a lane ends with four adjacent outputs of one token.  The workgroups of one head and
// token range run side by side on one XCD and share the rows through its L2; one more workgroup
// per range turns the rotary part.
constexpr int HG_BN = 64;

template <typename T, int KS>
__global__ __launch_bounds__(256, 2) void head_gemm_mfma_kernel(HeadGemm a, int groups, int nz,
                                                                int units) {
  typedef typename Vec8<T>::type V8;
  const int nza = nz + (a.rot != nullptr ? 1 : 0);
  const int xcd = blockIdx.x & 7, slot = blockIdx.x >> 3;
  const int z = slot % nza, u = (slot / nza) * 8 + xcd;
  if (u >= units) return;
  const int h = u / groups, g = u - h * groups;
  if (z == nz) {
    rotate_rows<T>(a, h, g * 256 + threadIdx.x, groups * 256);
    return;
  }
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, qd = lane >> 4;
  const T* w = static_cast<const T*>(a.w) + (int64_t)h * a.N * a.K;
  const T* x = static_cast<const T*>(a.x) + h * a.xh;
  T* out = static_cast<T*>(a.out) + h * a.oh;
  const int n0 = z * HG_BN, nks = (a.K + 31) >> 5;
  V8 wf[4][KS];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int n = min(n0 + 16 * j + r16, a.N - 1);
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      Pack8<T> p;
      p.u = u32x4{0u, 0u, 0u, 0u};
      if (32 * s + 8 * qd < a.K)
        p.u = *reinterpret_cast<const u32x4*>(w + (int64_t)n * a.K + 32 * s + 8 * qd);
      wf[j][s] = p.v;
    }
  }
  const int ntiles = (a.T + 15) >> 4;
  for (int tile = g * 4 + wave; tile < ntiles; tile += groups * 4) {
    const int t = tile * 16 + r16;
    const T* xr = x + (int64_t)min(t, a.T - 1) * a.xs;
    V8 xf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      Pack8<T> p;
      p.u = u32x4{0u, 0u, 0u, 0u};
      if (32 * s + 8 * qd < a.K) p.u = *reinterpret_cast<const u32x4*>(xr + 32 * s + 8 * qd);
      xf[s] = p.v;
    }
    T* orow = out + (int64_t)t * a.os;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s)
        if (s < nks) acc = mfma16x16x32(wf[j][s], xf[s], acc);
      const int n = n0 + 16 * j + 4 * qd;
      if (t < a.T && n < a.N) {
        Pack4<T> o;
#pragma unroll
        for (int i = 0; i < 4; ++i) o.h[i] = from_f<T>(acc[i]);
        *reinterpret_cast<u32x2*>(orow + n) = o.u;
      }
    }
  }
}

// Any type and sizes: a workgroup per (token, head), the row in LDS, an output per thread.
template <typename T>
__global__ __launch_bounds__(256) void head_gemm_any_kernel(HeadGemm a) {
  extern __shared__ float xl[];
  const int t = blockIdx.x, h = blockIdx.y;
  const T* x = static_cast<const T*>(a.x) + (int64_t)t * a.xs + h * a.xh;
  const T* w = static_cast<const T*>(a.w) + (int64_t)h * a.N * a.K;
  T* out = static_cast<T*>(a.out) + (int64_t)t * a.os + h * a.oh;
  for (int k = threadIdx.x; k < a.K; k += 256) xl[k] = to_f(x[k]);
  __syncthreads();
  for (int n = threadIdx.x; n < a.N; n += 256) {
    const T* wr = w + (int64_t)n * a.K;
    float acc = 0.f;
    for (int k = 0; k < a.K; ++k) acc += xl[k] * to_f(wr[k]);
    out[n] = from_f<T>(acc);
  }
  if (a.rot != nullptr) {
    const int half = a.r >> 1;
    int64_t pos = a.positions[t];
    if (pos < 0) pos = 0;
    if (pos >= a.table_rows) pos = a.table_rows - 1;
    const float* cs = a.table + pos * a.r;
    const T* src = static_cast<const T*>(a.rot) + (int64_t)t * a.rs + h * a.rh;
    for (int p = threadIdx.x; p < half; p += 256) {
      float oa, ob;
      neox_rot(to_f(src[2 * p]), to_f(src[2 * p + 1]), cs[p], cs[half + p], oa, ob);
      out[a.N + 2 * p] = from_f<T>(oa);
      out[a.N + 2 * p + 1] = from_f<T>(ob);
    }
  }
}

template <typename T>
void head_gemm_fast(const HeadGemm& a, hipStream_t s) {
  const int nz = (a.N + HG_BN - 1) / HG_BN, nza = nz + (a.rot != nullptr ? 1 : 0);
  const int per = (a.T + 63) / 64;                  // token ranges of one tile per wave
  // about 2048 workgroups when there are many tokens: the weights are loaded once per workgroup
  const int want = std::max(1, 2048 / (a.H * nza));
  const int groups = std::min(per, want), units = groups * a.H;
  const int grid = (units + 7) / 8 * 8 * nza;
  if (a.K <= 128) head_gemm_mfma_kernel<T, 4><<<grid, 256, 0, s>>>(a, groups, nz, units);
  else head_gemm_mfma_kernel<T, 8><<<grid, 256, 0, s>>>(a, groups, nz, units);
}

}  // namespace

void launch_latent_down_store(int dtype, void* cq, float* gate, const void* proj, int64_t ps,
                              const int64_t* positions, const float* table, int table_rows,
                              const float* qw, const float* kw, float eps, void* cache,
                              const int64_t* slots, int64_t cache_rows, int T_, int qr, int rank,
                              int r, int gates, hipStream_t s) {
  if (T_ <= 0) return;
  KGC_DISPATCH_T(dtype, latent_down_store_kernel<T><<<T_, 256, 0, s>>>(
      (T*)cq, gate, (const T*)proj, ps, positions, table, table_rows, qw, kw, eps, (T*)cache, slots,
      cache_rows, qr, rank, r, gates));
}

void launch_head_gemm(int dtype, HeadGemm a, hipStream_t s) {
  if (a.T <= 0) return;
  auto al = [](const void* p, int n) { return reinterpret_cast<uintptr_t>(p) % n == 0; };
  const bool fast = dtype != DT_F32 && a.K % 8 == 0 && a.K <= 256 && a.N % 4 == 0 &&
                    a.xs % 8 == 0 && a.xh % 8 == 0 && a.os % 4 == 0 && a.oh % 4 == 0 &&
                    al(a.x, 16) && al(a.w, 16) && al(a.out, 8);
  if (fast) {
    if (dtype == DT_BF16) head_gemm_fast<bf16>(a, s);
    else head_gemm_fast<f16>(a, s);
    return;
  }
  KGC_DISPATCH_T(dtype, head_gemm_any_kernel<T><<<dim3(a.T, a.H), 256, a.K * sizeof(float), s>>>(a));
}

}  // namespace kgc
