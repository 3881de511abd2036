// The gated delta rule with a decay per key channel, over per-sequence state slots, all fp32
// past the projections:
//   delta_gates         the second projections of the decay and output-gate bottlenecks in one
//                       launch; decay = exp(neg_a softplus(. + dt_bias)) in fp32
//   channel_delta_scan  S = diag(g) S;  u = beta (v - S^T k);  S += k u^T;  o = S^T q
//                       (q, k made unit vectors, q times d^-1/2)
// A step's sequences are its prefill chunks (rows [qsl[i], qsl[i+1]), first position
// seq_lens[i] - rows) followed by its decode rows (one row each, position ctx_lens - 1).  A
// chunk that starts at position 0 starts from zero state; a slot < 0 is a padding row and
// gives zeros.  Prefill chunks and decode rows run the same code, token by token, so a
// position's result does not depend on how the prompt was cut.
//
// Scan layout: grid (step sequences, heads, column tiles), four waves.  A wave owns 16 columns
// of S [d, V] (4 when few long sequences have to cover the chip); lane = column * row groups +
// row group, and a lane keeps the RPT consecutive rows rg RPT .. of its column in registers for
// the whole chunk.  The row groups of a column are adjacent lanes of one 16-lane row, so both
// sums over key channels end in data-parallel-primitive adds inside the vector ALU: a token
// costs no barrier and no LDS round trip.  Tokens are staged in LDS 16 at a time; the next
// block's loads are in flight while the current one is walked.
#include "common.h"
#include "launch.h"

namespace kgc {

namespace {

constexpr int NT = 256;
constexpr int TB = 16;             // tokens staged per block

__device__ __forceinline__ float softplus_f(float x) {
  return x > 20.f ? x : log1pf(expf(x));
}
__device__ __forceinline__ float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }

template <int CTRL>
__device__ __forceinline__ float dpp_f(float v) {
  return __builtin_bit_cast(
      float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}

// sum over groups of N adjacent lanes (16: a lane row, rotations; 4: a quad, permutations);
// every lane of the group gets the same value
template <int N>
__device__ __forceinline__ float group_sum(float v) {
  if constexpr (N == 16) {
    v += dpp_f<0x128>(v);          // row_ror:8, 4, 2, 1
    v += dpp_f<0x124>(v);
    v += dpp_f<0x122>(v);
    v += dpp_f<0x121>(v);
  } else {
    static_assert(N == 4, "quads or lane rows");
    v += dpp_f<0xB1>(v);           // quad_perm [1, 0, 3, 2]
    v += dpp_f<0x4E>(v);           // quad_perm [2, 3, 0, 1]
  }
  return v;
}

// LDS place of key channel r when a lane owns RPT consecutive ones: the row groups are padded
// by four floats so that their 16-byte reads fall into different banks
template <int RPT>
__device__ __forceinline__ int lrow(int r) { return r + 4 * (r / RPT); }

// ---- the two second projections -------------------------------------------------------------
// low [T, ra + rg] (row stride ls), a2 [Nd, ra], g2 [Ng, rg]; decay fp32 [T, Nd], gate [T, Ng].
// 16-bit types: one wave per 16 rows x 64 columns on the matrix cores (the weight rows are the
// A operand, so a lane's four results are adjacent columns of one row).  ra, rg: multiples of 32.
template <typename T>
__global__ __launch_bounds__(NT) void delta_gates_mfma_kernel(
    float* __restrict__ decay, T* __restrict__ gate, const T* __restrict__ low, int64_t ls,
    const T* __restrict__ a2, const T* __restrict__ g2, const float* __restrict__ neg_a,
    const float* __restrict__ dt_bias, int T_, int Nd, int Ng, int ra, int rg, int nbd) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, qd = lane >> 4;
  const int t0 = (blockIdx.x * 4 + wave) * 16;
  if (t0 >= T_) return;
  const bool isd = (int)blockIdx.y < nbd;              // decay columns, then gate columns
  const int n0 = (isd ? blockIdx.y : blockIdx.y - nbd) * 64;
  const int N = isd ? Nd : Ng, R = isd ? ra : rg;
  const T* W = isd ? a2 : g2;
  const int t = t0 + r16;
  const T* lrp = low + (int64_t)min(t, T_ - 1) * ls + (isd ? 0 : ra) + 8 * qd;
  f32x4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < R; k += 32) {
    Pack8<T> lf;
    lf.u = *reinterpret_cast<const u32x4*>(lrp + k);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      Pack8<T> wf;
      const int n = min(n0 + 16 * j + r16, N - 1);     // clamped: rows past N are not stored
      wf.u = *reinterpret_cast<const u32x4*>(W + (int64_t)n * R + k + 8 * qd);
      acc[j] = mfma16x16x32(wf.v, lf.v, acc[j]);
    }
  }
  if (t >= T_) return;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int n = n0 + 16 * j + 4 * qd;
    if (isd) {
      float v[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int c = min(n + i, N - 1);
        v[i] = expf(neg_a[c] * softplus_f(acc[j][i] + dt_bias[c]));
      }
      float* o = decay + (int64_t)t * N + n;
      if (n + 3 < N && (N & 3) == 0) {
        *reinterpret_cast<float4*>(o) = make_float4(v[0], v[1], v[2], v[3]);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (n + i < N) o[i] = v[i];
      }
    } else {
      T* o = gate + (int64_t)t * N + n;
      if (n + 3 < N && (N & 3) == 0) {
        Pack4<T> p;
#pragma unroll
        for (int i = 0; i < 4; ++i) p.h[i] = from_f<T>(acc[j][i]);
        *reinterpret_cast<u32x2*>(o) = p.u;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (n + i < N) o[i] = from_f<T>(acc[j][i]);
      }
    }
  }
}

// any element type and alignment: one thread per output
template <typename T>
__global__ __launch_bounds__(NT) void delta_gates_any_kernel(
    float* __restrict__ decay, T* __restrict__ gate, const T* __restrict__ low, int64_t ls,
    const T* __restrict__ a2, const T* __restrict__ g2, const float* __restrict__ neg_a,
    const float* __restrict__ dt_bias, int Nd, int Ng, int ra, int rg) {
  const int64_t t = blockIdx.x;
  const int c = blockIdx.y * NT + threadIdx.x;
  if (c >= Nd + Ng) return;
  const bool isd = c < Nd;
  const int n = isd ? c : c - Nd, R = isd ? ra : rg;
  const T* w = (isd ? a2 : g2) + (int64_t)n * R;
  const T* l = low + t * ls + (isd ? 0 : ra);
  float acc = 0.f;
  for (int k = 0; k < R; ++k) acc += to_f(l[k]) * to_f(w[k]);
  if (isd) decay[t * Nd + n] = expf(neg_a[n] * softplus_f(acc + dt_bias[n]));
  else gate[t * Ng + n] = from_f<T>(acc);
}

// ---- the scan ---------------------------------------------------------------------------------
// qkv fp32 [T, 2 G d + H V] = q | k | v; b [T, H] (row stride bstr) write-strength
// pre-activations; decay fp32 [T, H d].  With S_0 the state before the token, G = diag(g) S_0:
//   u = beta (v - G^T k),  S = G + k u^T,  o = G^T q + (k . q) u
// so both sums run over G in one pass; the unit-vector factors of q and k are per-token scalars.
template <typename T, int RPT, int NRG>
__global__ __launch_bounds__(NT) void channel_delta_scan_kernel(
    float* __restrict__ out, const float* __restrict__ qkv, const T* __restrict__ b, int64_t bstr,
    const float* __restrict__ decay, float* __restrict__ S, const int* __restrict__ qsl,
    const int* __restrict__ seq_lens, const int* __restrict__ ctx_lens,
    const int* __restrict__ slots, int P, int Tp, int H, int G, int d, int V, int num_slots) {
  constexpr int CW = 64 / NRG, CT = CW * (NT / 64);   // columns per wave / per workgroup
  constexpr int RP = NRG * RPT, RPS = RP + 4 * NRG;   // rows (padded), LDS floats per vector
  constexpr int NE = TB * RP / NT;                    // staged elements per thread and vector
  constexpr int NV = (TB * CT + NT - 1) / NT;
  extern __shared__ float lds[];
  float* ks = lds;                   // [TB][RPS]
  float* qs = ks + TB * RPS;         // [TB][RPS]
  float* gs = qs + TB * RPS;         // [TB][RPS]
  float* vs = gs + TB * RPS;         // [TB][CT]
  float* sc = vs + TB * CT;          // [TB][4]: |k|^-1, |q|^-1 d^-1/2, k . q, write strength
  const int s = blockIdx.x, h = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, rg = lane & (NRG - 1);
  const int lc = wave * CW + lane / NRG, col = blockIdx.z * CT + lc;
  const bool colok = col < V;
  int start, len, pos0;
  if (s < P) {
    start = qsl[s];
    len = qsl[s + 1] - start;
    pos0 = seq_lens[s] - len;
  } else {
    start = Tp + (s - P);
    len = 1;
    pos0 = ctx_lens[s - P] - 1;
  }
  const int slot = slots[s];
  const int64_t ow = (int64_t)H * V;
  if (slot < 0 || slot >= num_slots || pos0 < 0 || len <= 0) {
    if (rg == 0 && colok)
      for (int t = 0; t < len; ++t) out[(int64_t)(start + t) * ow + h * V + col] = 0.f;
    return;
  }
  const int g = h / (H / G);
  const int64_t cw = (int64_t)2 * G * d + (int64_t)H * V, dw = (int64_t)H * d;
  const int qoff = g * d, koff = G * d + g * d, voff = 2 * G * d + h * V + blockIdx.z * CT;
  float* Sp = S + ((int64_t)slot * H + h) * d * V;
  float Sr[RPT];
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg * RPT + i;
    Sr[i] = (pos0 != 0 && r < d && colok) ? Sp[(int64_t)r * V + col] : 0.f;
  }
  const float qscale = 1.f / sqrtf((float)d);
  const int vcols = V - blockIdx.z * CT;
  // the block of tokens t0 .. of this thread's staging slots (zeros past the chunk / the rows)
  float rk[NE], rq[NE], rd[NE], rv[NV], rb = 0.f;
  auto fetch = [&](int t0) {
    const int nb = min(TB, len - t0);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = threadIdx.x + i * NT, tb = e / RP, r = e & (RP - 1);
      rk[i] = rq[i] = rd[i] = 0.f;
      if (tb < nb && r < d) {
        const int64_t t = start + t0 + tb;
        const float* row = qkv + t * cw;
        rk[i] = row[koff + r];
        rq[i] = row[qoff + r];
        rd[i] = decay[t * dw + h * d + r];
      }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = threadIdx.x + i * NT, tb = e / CT, c = e & (CT - 1);
      rv[i] = (tb < nb && c < vcols) ? qkv[(int64_t)(start + t0 + tb) * cw + voff + c] : 0.f;
    }
    // write strengths: the lane that keeps token wave * 4 + lane / 16 in the norm step
    const int tb = wave * 4 + (lane >> 4);
    if (tb < nb) rb = to_f(b[(int64_t)(start + t0 + tb) * bstr + h]);
  };
  fetch(0);
  for (int t0 = 0; t0 < len; t0 += TB) {
    const int nb = min(TB, len - t0);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = threadIdx.x + i * NT, tb = e / RP, r = e & (RP - 1);
      if (tb < nb) {
        const int a = tb * RPS + lrow<RPT>(r);
        ks[a] = rk[i];
        qs[a] = rq[i];
        gs[a] = rd[i];
      }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = threadIdx.x + i * NT;
      if (e < nb * CT) vs[e] = rv[i];
    }
    __syncthreads();
    {
      // 16 lanes per token: squared lengths and k . q
      const int tb = wave * 4 + (lane >> 4), sub = lane & 15;
      float sq = 0.f, sk = 0.f, kq = 0.f;
      if (tb < nb) {
#pragma unroll
        for (int i = 0; i < RP / 16; ++i) {
          const int a = tb * RPS + lrow<RPT>(sub + 16 * i);
          const float kv = ks[a], qv = qs[a];
          sq += qv * qv;
          sk += kv * kv;
          kq += kv * qv;
        }
      }
      sq = group_sum<16>(sq);
      sk = group_sum<16>(sk);
      kq = group_sum<16>(kq);
      if (sub == 0 && tb < nb) {
        const float kn = 1.f / sqrtf(sk + 1e-6f), qn = qscale / sqrtf(sq + 1e-6f);
        *reinterpret_cast<float4*>(sc + 4 * tb) = make_float4(kn, qn, kq * kn * qn, sigmoid_f(rb));
      }
    }
    __syncthreads();
    if (t0 + TB < len) fetch(t0 + TB);
    for (int tb = 0; tb < nb; ++tb) {
      const float4 c4 = *reinterpret_cast<const float4*>(sc + 4 * tb);
      const float vv = vs[tb * CT + lc];
      const int base = tb * RPS + rg * (RPT + 4);
      float k0 = 0.f, k1 = 0.f, q0 = 0.f, q1 = 0.f, kr[RPT];
#pragma unroll
      for (int i = 0; i < RPT; i += 4) {
        const float4 gv = *reinterpret_cast<const float4*>(gs + base + i);
        const float4 kv = *reinterpret_cast<const float4*>(ks + base + i);
        const float4 qv = *reinterpret_cast<const float4*>(qs + base + i);
        Sr[i] *= gv.x;
        Sr[i + 1] *= gv.y;
        Sr[i + 2] *= gv.z;
        Sr[i + 3] *= gv.w;
        k0 += Sr[i] * kv.x;
        k1 += Sr[i + 1] * kv.y;
        k0 += Sr[i + 2] * kv.z;
        k1 += Sr[i + 3] * kv.w;
        q0 += Sr[i] * qv.x;
        q1 += Sr[i + 1] * qv.y;
        q0 += Sr[i + 2] * qv.z;
        q1 += Sr[i + 3] * qv.w;
        kr[i] = kv.x;
        kr[i + 1] = kv.y;
        kr[i + 2] = kv.z;
        kr[i + 3] = kv.w;
      }
      const float sk = group_sum<NRG>(k0 + k1), sq = group_sum<NRG>(q0 + q1);
      const float u = c4.w * (vv - c4.x * sk), ku = c4.x * u;
#pragma unroll
      for (int i = 0; i < RPT; ++i) Sr[i] += kr[i] * ku;
      if (rg == 0 && colok)
        out[(int64_t)(start + t0 + tb) * ow + h * V + col] = c4.y * sq + c4.z * u;
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i) {
    const int r = rg * RPT + i;
    if (r < d && colok) Sp[(int64_t)r * V + col] = Sr[i];
  }
}

}  // namespace

#define KGC_CD_DISPATCH_T(dtype, ...)                       \
  do {                                                      \
    if ((dtype) == DT_BF16) { typedef bf16 T; __VA_ARGS__; } \
    else if ((dtype) == DT_F16) { typedef f16 T; __VA_ARGS__; } \
    else { typedef float T; __VA_ARGS__; }                  \
  } while (0)

void launch_delta_gates(int dtype, float* decay, void* gate, const void* low, int64_t ls,
                        const void* a2, const void* g2, const float* neg_a, const float* dt_bias,
                        int T_, int Nd, int Ng, int ra, int rg, hipStream_t s) {
  if (T_ <= 0) return;
  const bool mfma = dtype != DT_F32 && ra % 32 == 0 && rg % 32 == 0 && ls % 8 == 0 &&
                    reinterpret_cast<uintptr_t>(low) % 16 == 0;
  if (mfma) {
    const int nbd = (Nd + 63) / 64;
    const dim3 grid((T_ + 63) / 64, nbd + (Ng + 63) / 64);
    if (dtype == DT_BF16)
      delta_gates_mfma_kernel<bf16><<<grid, NT, 0, s>>>(
          decay, (bf16*)gate, (const bf16*)low, ls, (const bf16*)a2, (const bf16*)g2, neg_a,
          dt_bias, T_, Nd, Ng, ra, rg, nbd);
    else
      delta_gates_mfma_kernel<f16><<<grid, NT, 0, s>>>(
          decay, (f16*)gate, (const f16*)low, ls, (const f16*)a2, (const f16*)g2, neg_a, dt_bias,
          T_, Nd, Ng, ra, rg, nbd);
    return;
  }
  const dim3 grid(T_, (Nd + Ng + NT - 1) / NT);
  KGC_CD_DISPATCH_T(dtype, delta_gates_any_kernel<T><<<grid, NT, 0, s>>>(
      decay, (T*)gate, (const T*)low, ls, (const T*)a2, (const T*)g2, neg_a, dt_bias, Nd, Ng, ra,
      rg));
}

int channel_delta_max_rows() { return 256; }

void launch_channel_delta_scan(int dtype, float* out, const float* qkv, const void* b,
                               int64_t bstr, const float* decay, float* S, const int* qsl,
                               const int* seq_lens, const int* ctx_lens, const int* slots, int P,
                               int D, int Tp, int H, int G, int d, int V, int num_slots,
                               hipStream_t s) {
  if (P + D <= 0) return;
  // columns per wave: 16 when that already gives the chip two workgroups per CU, else 4, so
  // that few long sequences still spread over the chip
  const bool narrow = V <= 4 || (int64_t)(P + D) * H * ((V + 63) / 64) < 512;
  const int nrg = narrow ? 16 : 4, ct = narrow ? 16 : 64;
  int rp = narrow ? 64 : 16;
  while (rp < d) rp <<= 1;
  const dim3 grid(P + D, H, (V + ct - 1) / ct);
  const size_t lds = sizeof(float) * (size_t)(3 * TB * (rp + 4 * nrg) + TB * ct + TB * 4);
#define KGC_CDS(R, N)                                                                        \
  KGC_CD_DISPATCH_T(dtype, channel_delta_scan_kernel<T, R, N><<<grid, NT, lds, s>>>(         \
      out, qkv, (const T*)b, bstr, decay, S, qsl, seq_lens, ctx_lens, slots, P, Tp, H, G, d, V, \
      num_slots))
  if (narrow) {
    if (rp <= 64) KGC_CDS(4, 16);
    else if (rp == 128) KGC_CDS(8, 16);
    else KGC_CDS(16, 16);
  } else {
    if (rp <= 16) KGC_CDS(4, 4);
    else if (rp == 32) KGC_CDS(8, 4);
    else if (rp == 64) KGC_CDS(16, 4);
    else if (rp == 128) KGC_CDS(32, 4);
    else KGC_CDS(64, 4);
  }
#undef KGC_CDS
}

}  // namespace kgc
