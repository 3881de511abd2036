// Hyper-connections: S residual streams per token, fp32 [rows, S, W].  One pass per sublayer:
//   y = the sublayer's result (sum of up to two addends, each the sum of a few rows per token)
//   x_t = sum_s mix[s, t] src_s + ow[t] y            (all streams from the old ones)
//   out = u / rms(u) * w,  u = sum_s iw[s] x_s       (w null: u; out null: none)
// so the streams are read once and written once, and the next sublayer's input, its norm and the
// combination of expert rows need no pass of their own.  One workgroup per row; a thread owns
// columns threadIdx.x * VEC + k * 256 VEC of every stream, which makes in-place updates safe.
#include "common.h"
#include "launch.h"

namespace kgc {

namespace {

constexpr int HN = 256;

template <typename T, int VEC>
__device__ __forceinline__ void ldv(const T* p, float (&v)[VEC]) {
  if constexpr (VEC == 1) {
    v[0] = to_f(p[0]);
  } else if constexpr (std::is_same_v<T, float>) {
    const float4 t = *reinterpret_cast<const float4*>(p);
    v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
  } else {
    Pack4<T> t;
    t.u = *reinterpret_cast<const u32x2*>(p);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = to_f(t.h[e]);
  }
}
template <typename T, int VEC>
__device__ __forceinline__ void stv(T* p, const float (&v)[VEC]) {
  if constexpr (VEC == 1) {
    p[0] = from_f<T>(v[0]);
  } else if constexpr (std::is_same_v<T, float>) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  } else {
    Pack4<T> t;
#pragma unroll
    for (int e = 0; e < 4; ++e) t.h[e] = from_f<T>(v[e]);
    *reinterpret_cast<u32x2*>(p) = t.u;
  }
}

// y[c ..] of a token: every addend's rows, and its partial sums when it is fp32 slices
template <typename T, int VEC>
__device__ __forceinline__ void add_rows(const HyperAdds& ad, int64_t row, int W, int c,
                                         float (&y)[VEC]) {
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    if (ad.a[j] == nullptr) continue;
    for (int r = 0; r < ad.k[j]; ++r) {
      const int64_t o = (row * ad.k[j] + r) * W + c;
      float v[VEC];
      if (ad.slices[j] == 0) {
        ldv<T, VEC>(static_cast<const T*>(ad.a[j]) + o, v);
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[e] += v[e];
      } else {
        for (int z = 0; z < ad.slices[j]; ++z) {
          ldv<float, VEC>(static_cast<const float*>(ad.a[j]) + z * ad.ss[j] + o, v);
#pragma unroll
          for (int e = 0; e < VEC; ++e) y[e] += v[e];
        }
      }
    }
  }
}

// SM: streams the loops are unrolled for (exact up to 4, an upper bound beyond).  NC > 0: the
// thread's columns of u stay in registers (W <= NC * 256 * VEC); NC = 0: in LDS.
template <typename T, typename O, int SM, int VEC, int NC>
__global__ __launch_bounds__(HN) void hyper_norm_kernel(
    O* __restrict__ out, const float* src, int64_t srow, int64_t sstream, float* dst,
    HyperAdds ad, const float* __restrict__ mix, const float* __restrict__ ow,
    const float* __restrict__ iw, const float* __restrict__ w, int S, int W, float eps) {
  extern __shared__ float us[];
  __shared__ float scratch[HN / 64];
  const int64_t row = blockIdx.x;
  const float* sr = src + row * srow;
  float* dr = dst != nullptr ? dst + row * S * W : nullptr;
  auto in = [&](int s) { return SM <= 4 || s < S; };
  // one column group: the new streams, stored when wanted; -> u
  auto group = [&](int c, const float (&x)[SM][VEC], float (&u)[VEC]) {
    float y[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = u[e] = 0.f;
    if (mix != nullptr) {
      add_rows<T, VEC>(ad, row, W, c, y);
#pragma unroll
      for (int t = 0; t < SM; ++t) {
        if (!in(t)) continue;
        float v[VEC];
        const float o = ow[t];
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = o * y[e];
#pragma unroll
        for (int s = 0; s < SM; ++s) {
          if (!in(s)) continue;
          const float m = mix[s * S + t];
#pragma unroll
          for (int e = 0; e < VEC; ++e) v[e] += m * x[s][e];
        }
        if (dr != nullptr) stv<float, VEC>(dr + (int64_t)t * W + c, v);
        const float i = iw[t];
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] += i * v[e];
      }
    } else {
#pragma unroll
      for (int s = 0; s < SM; ++s) {
        if (!in(s)) continue;
        const float i = iw[s];
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] += i * x[s][e];
      }
    }
  };
  auto load = [&](int c, float (&x)[SM][VEC]) {
#pragma unroll
    for (int s = 0; s < SM; ++s)
      if (in(s)) ldv<float, VEC>(sr + s * sstream + c, x[s]);
  };
  float ss = 0.f;
  if constexpr (NC > 0) {
    float x[NC][SM][VEC], u[NC][VEC];
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = (threadIdx.x + k * HN) * VEC;
      if (c < W) load(c, x[k]);
    }
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = (threadIdx.x + k * HN) * VEC;
      if (c < W) {
        group(c, x[k], u[k]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) ss += u[k][e] * u[k][e];
      }
    }
    if (out == nullptr) return;
    float r = 1.f;
    if (w != nullptr) {
      ss = block_sum<HN>(ss, scratch);
      r = 1.f / sqrtf(ss / (float)W + eps);
    }
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = (threadIdx.x + k * HN) * VEC;
      if (c < W) {
        if (w != nullptr) {
          float wv[VEC];
          ldv<float, VEC>(w + c, wv);
#pragma unroll
          for (int e = 0; e < VEC; ++e) u[k][e] *= r * wv[e];
        }
        stv<O, VEC>(out + row * W + c, u[k]);
      }
    }
  } else {
    for (int c = threadIdx.x * VEC; c < W; c += HN * VEC) {
      float x[SM][VEC], u[VEC];
      load(c, x);
      group(c, x, u);
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        us[c + e] = u[e];
        ss += u[e] * u[e];
      }
    }
    if (out == nullptr) return;
    float r = 1.f;
    if (w != nullptr) {
      ss = block_sum<HN>(ss, scratch);
      r = 1.f / sqrtf(ss / (float)W + eps);
    }
    for (int c = threadIdx.x * VEC; c < W; c += HN * VEC) {      // (the thread's own columns)
      float u[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) u[e] = us[c + e] * (w != nullptr ? r * w[c + e] : 1.f);
      stv<O, VEC>(out + row * W + c, u);
    }
  }
}

template <typename T, typename O>
void hyper_dispatch(O* out, const float* src, int64_t srow, int64_t sstream, float* dst,
                    const HyperAdds& ad, const float* mix, const float* ow, const float* iw,
                    const float* w, int rows, int S, int W, float eps, bool vec, hipStream_t s) {
#define KGC_HY(SM, V, N)                                                                    \
  hyper_norm_kernel<T, O, SM, V, N><<<rows, HN, (N) > 0 ? 0 : W * sizeof(float), s>>>(      \
      out, src, srow, sstream, dst, ad, mix, ow, iw, w, S, W, eps)
#define KGC_HY_W(SM)                              \
  do {                                            \
    if (!vec) KGC_HY(SM, 1, 0);                   \
    else if (W <= 4 * HN) KGC_HY(SM, 4, 1);       \
    else if (W <= 8 * HN) KGC_HY(SM, 4, 2);       \
    else if (W <= 16 * HN) KGC_HY(SM, 4, 4);      \
    else KGC_HY(SM, 4, 0);                        \
  } while (0)
  if (S == 1) KGC_HY_W(1);
  else if (S == 2) KGC_HY_W(2);
  else if (S == 3) KGC_HY_W(3);
  else if (S == 4) KGC_HY_W(4);
  else if (S <= 8 && vec) KGC_HY(8, 4, 0);
  else KGC_HY(32, 1, 0);
#undef KGC_HY_W
#undef KGC_HY
}

}  // namespace

int hyper_max_streams() { return 32; }

void launch_hyper_norm(int dtype, int out_dtype, void* out, const float* src, int64_t srow,
                       int64_t sstream, float* dst, HyperAdds ad, const float* mix,
                       const float* ow, const float* iw, const float* w, int rows, int S, int W,
                       float eps, hipStream_t s) {
  if (rows <= 0) return;
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = W % 4 == 0 && srow % 4 == 0 && sstream % 4 == 0 && al(src) && al(dst) &&
                   al(out) && al(w) && al(ad.a[0]) && al(ad.a[1]);
#define KGC_HY_D(T, O) \
  hyper_dispatch<T, O>((O*)out, src, srow, sstream, dst, ad, mix, ow, iw, w, rows, S, W, eps, vec, s)
  const bool f32out = out == nullptr || out_dtype == DT_F32;
  if (dtype == DT_BF16) {
    if (f32out) KGC_HY_D(bf16, float); else KGC_HY_D(bf16, bf16);
  } else if (dtype == DT_F16) {
    if (f32out) KGC_HY_D(f16, float); else KGC_HY_D(f16, f16);
  } else {
    KGC_HY_D(float, float);
  }
#undef KGC_HY_D
}

}  // namespace kgc
