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
// Scan layout: grid (prefill sequences, heads, column tiles), four waves.  A wave owns 4 CPL
// columns of S [d, V]; lane = column lane * 16 + row group, and a lane keeps RPT consecutive rows
// of CPL columns in registers for the whole chunk.  The row groups of a column are the 16 lanes
// of one lane row, so both sums over key channels end in rotations inside the vector ALU: a token
// costs no barrier and no LDS round trip.  Tokens are staged in LDS 16 at a time; the next
// block's loads are in flight while the current one is walked, and the next token's LDS reads
// while the current one is computed.  CPL columns share a lane's k, q and decay reads; few long
// sequences take a smaller CPL so that they still spread over the chip.
//
// Decode layout: grid (decode rows, heads, 64-column tiles): a state row is read and written 256
// bytes at a time (16 lanes x 4 columns), all of a lane's rows in flight at once; sums over rows
// cross lane rows by swaps and waves through LDS.
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

// sum over a row of 16 adjacent lanes; every lane of the row gets the same value
__device__ __forceinline__ float row_sum(float v) {
  v += dpp_f<0x128>(v);            // row_ror:8, 4, 2, 1
  v += dpp_f<0x124>(v);
  v += dpp_f<0x122>(v);
  v += dpp_f<0x121>(v);
  return v;
}

// sum over the four lane rows of a wave (lanes l, l ^ 16, l ^ 32, l ^ 48)
__device__ __forceinline__ float across_rows(float v) {
  const unsigned u = __builtin_bit_cast(unsigned, v);
  auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  v = __builtin_bit_cast(float, (unsigned)a[0]) + __builtin_bit_cast(float, (unsigned)a[1]);
  const unsigned w = __builtin_bit_cast(unsigned, v);
  auto b = __builtin_amdgcn_permlane32_swap(w, w, false, false);
  return __builtin_bit_cast(float, (unsigned)b[0]) + __builtin_bit_cast(float, (unsigned)b[1]);
}

// LDS place of key channel r when a lane owns RPT consecutive ones: the row groups are padded
// by four floats so that their 16-byte reads fall into different banks
template <int RPT>
__device__ __forceinline__ int lrow(int r) { return r + 4 * (r / RPT); }

// ---- the two second projections -------------------------------------------------------------
// low [T, ra + rg] (row stride ls), a2 [Nd, ra], g2 [Ng, rg]; decay fp32 [T, Nd], gate [T, Ng].
// 16-bit types: a wave keeps the weight fragments of 64 columns in registers (up to KMAX steps
// of 32) and walks `tiles` tiles of 16 rows on the matrix cores, the next tile's rows in flight;
// the four waves of a workgroup take adjacent columns of the same rows.  The weight rows are the
// A operand, so a lane's four results are adjacent columns of one row.  ra, rg: multiples of 32,
// at most 32 KMAX.
template <typename T, int KMAX>
__global__ __launch_bounds__(NT) void delta_gates_mfma_kernel(
    float* __restrict__ decay, T* __restrict__ gate, const T* __restrict__ low, int64_t ls,
    const T* __restrict__ a2, const T* __restrict__ g2, const float* __restrict__ neg_a,
    const float* __restrict__ dt_bias, int T_, int Nd, int Ng, int ra, int rg, int nbd, int tiles) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, qd = lane >> 4;
  const int strip = blockIdx.y * 4 + wave;             // decay columns, then gate columns
  const bool isd = strip < nbd;
  const int n0 = (isd ? strip : strip - nbd) * 64;
  const int N = isd ? Nd : Ng, R = isd ? ra : rg;
  const T* W = isd ? a2 : g2;
  if (n0 >= N) return;
  Pack8<T> wf[4][KMAX];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int n = min(n0 + 16 * j + r16, N - 1);       // clamped: rows past N are not stored
#pragma unroll
    for (int k = 0; k < KMAX; ++k)
      if (32 * k < R) wf[j][k].u = *reinterpret_cast<const u32x4*>(W + (int64_t)n * R + 32 * k + 8 * qd);
  }
  float na[4][4], db[4][4];
#pragma unroll
  for (int j = 0; j < 4; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = min(n0 + 16 * j + 4 * qd + i, N - 1);
      na[j][i] = isd ? neg_a[c] : 0.f;
      db[j][i] = isd ? dt_bias[c] : 0.f;
    }
  const T* lcol = low + (isd ? 0 : ra) + 8 * qd;
  const bool vec = (N & 3) == 0;
  Pack8<T> lf[KMAX];
  auto fetch = [&](int t0) {
    const T* p = lcol + (int64_t)min(t0 + r16, T_ - 1) * ls;
#pragma unroll
    for (int k = 0; k < KMAX; ++k)
      if (32 * k < R) lf[k].u = *reinterpret_cast<const u32x4*>(p + 32 * k);
  };
  fetch(blockIdx.x * tiles * 16);
  for (int m = 0; m < tiles; ++m) {
    const int t0 = (blockIdx.x * tiles + m) * 16;
    if (t0 >= T_) return;
    const int t = t0 + r16;
    f32x4 acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KMAX; ++k) {
      if (32 * k < R) {
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = mfma16x16x32(wf[j][k].v, lf[k].v, acc[j]);
      }
    }
    if (m + 1 < tiles) fetch(t0 + 16);
    if (t >= T_) continue;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + 16 * j + 4 * qd;
      if (isd) {
        float v[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          // ln(1 + e^z) on the hardware exponential and logarithm: its absolute error is that
          // of rounding 1 + e^z, no more than the rounding of a decay close to 1
          const float z = acc[j][i] + db[j][i];
          v[i] = __expf(na[j][i] * (z > 20.f ? z : __logf(1.f + __expf(z))));
        }
        float* o = decay + (int64_t)t * N + n;
        if (vec && n < N) {
          *reinterpret_cast<float4*>(o) = make_float4(v[0], v[1], v[2], v[3]);
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (n + i < N) o[i] = v[i];
        }
      } else {
        T* o = gate + (int64_t)t * N + n;
        if (vec && n < N) {
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
__device__ __forceinline__ void ld4(const float* p, float* v) {
  const float4 t = *reinterpret_cast<const float4*>(p);
  v[0] = t.x;
  v[1] = t.y;
  v[2] = t.z;
  v[3] = t.w;
}

// what one token needs in registers: a lane's decays, k and q, the token's scalars, its values
template <int RPT, int CPL>
struct TokenRegs {
  float g[RPT], k[RPT], q[RPT], c[4], v[CPL];
};

// row_sum of N independent values, step by step side by side
template <int N>
__device__ __forceinline__ void row_sums(float (&v)[N]) {
#pragma unroll
  for (int c = 0; c < N; ++c) v[c] += dpp_f<0x128>(v[c]);
#pragma unroll
  for (int c = 0; c < N; ++c) v[c] += dpp_f<0x124>(v[c]);
#pragma unroll
  for (int c = 0; c < N; ++c) v[c] += dpp_f<0x122>(v[c]);
#pragma unroll
  for (int c = 0; c < N; ++c) v[c] += dpp_f<0x121>(v[c]);
}

template <typename T, int RPT, int CPL>
__global__ __launch_bounds__(NT) void channel_delta_scan_kernel(
    float* __restrict__ out, const float* __restrict__ qkv, const T* __restrict__ b, int64_t bstr,
    const float* __restrict__ decay, float* __restrict__ S, const int* __restrict__ start_loc,
    const int* __restrict__ ctx, const int* __restrict__ slots, int row0, int H, int G, int d,
    int V, int num_slots) {
  constexpr int NRG = 16, CT = 4 * CPL * (NT / 64);   // row groups, columns per workgroup
  constexpr int RP = NRG * RPT, RPS = RP + 4 * NRG;   // rows (padded), LDS floats per vector
  constexpr int NE = TB * RP / NT;                    // staged elements per thread and vector
  constexpr int NV = TB * CT / NT;
  extern __shared__ float lds[];
  float* ks = lds;                   // [TB][RPS]
  float* qs = ks + TB * RPS;         // [TB][RPS]
  float* gs = qs + TB * RPS;         // [TB][RPS]
  float* vs = gs + TB * RPS;         // [TB][CT]
  float* sc = vs + TB * CT;          // [TB][4]: |k|^-1, |q|^-1 d^-1/2, k . q, write strength
  const int s = blockIdx.x, h = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, rg = lane & (NRG - 1);
  const int lc = (wave * 4 + (lane >> 4)) * CPL, col = blockIdx.z * CT + lc;
  // a chunk: rows [start_loc[s], start_loc[s + 1]), ctx[s] tokens up to its end; without
  // start_loc single rows (row0 + s, at position ctx[s] - 1)
  const int start = start_loc != nullptr ? start_loc[s] : row0 + s;
  const int len = start_loc != nullptr ? start_loc[s + 1] - start : 1;
  const int pos0 = ctx[s] - len, slot = slots[s];
  const int64_t ow = (int64_t)H * V;
  if (slot < 0 || slot >= num_slots || pos0 < 0 || len <= 0) {
    if (rg == 0)
      for (int t = 0; t < len; ++t)
        for (int c = 0; c < CPL; ++c)
          if (col + c < V) out[(int64_t)(start + t) * ow + h * V + col + c] = 0.f;
    return;
  }
  const int g = h / (H / G);
  const int64_t cw = (int64_t)2 * G * d + (int64_t)H * V, dw = (int64_t)H * d;
  const int qoff = g * d, koff = G * d + g * d, voff = 2 * G * d + h * V + blockIdx.z * CT;
  float* Sp = S + ((int64_t)slot * H + h) * d * V;
  float Sr[RPT][CPL];
#pragma unroll
  for (int i = 0; i < RPT; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const int r = rg * RPT + i;
      Sr[i][c] = (pos0 != 0 && r < d && col + c < V) ? Sp[(int64_t)r * V + col + c] : 0.f;
    }
  const float qscale = 1.f / sqrtf((float)d);
  const int vcols = V - blockIdx.z * CT;
  // the block of tokens t0 .. of this thread's staging slots
  float rk[NE], rq[NE], rd[NE], rv[NV], rb = 0.f;
  auto fetch = [&](int t0) {
    // (tokens past the chunk repeat its last one and are not used: no branch around a load)
    const int last = min(TB, len - t0) - 1;
    // wave-uniform bases and 32-bit lane offsets within the block
    const float* row = qkv + (int64_t)(start + t0) * cw;
    const float *kb = row + koff, *qb = row + qoff, *vb = row + voff;
    const float* gb = decay + (int64_t)(start + t0) * dw + h * d;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = threadIdx.x + i * NT, r = min(e & (RP - 1), d - 1), tb = min(e / RP, last);
      const unsigned o = (unsigned)(tb * (int)cw + r);
      rk[i] = kb[o];
      rq[i] = qb[o];
      rd[i] = gb[(unsigned)(tb * (int)dw + r)];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = threadIdx.x + i * NT, c = min(e & (CT - 1), vcols - 1);
      rv[i] = vb[(unsigned)(min(e / CT, last) * (int)cw + c)];
    }
    // write strengths: the lane that keeps token wave * 4 + lane / 16 in the norm step
    rb = to_f(b[(int64_t)(start + t0 + min(wave * 4 + (lane >> 4), last)) * bstr + h]);
  };
  fetch(0);
  for (int t0 = 0; t0 < len; t0 += TB) {
    const int nb = min(TB, len - t0);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int e = threadIdx.x + i * NT, r = e & (RP - 1);
      const int a = (e / RP) * RPS + lrow<RPT>(r);
      ks[a] = r < d ? rk[i] : 0.f;
      qs[a] = r < d ? rq[i] : 0.f;
      gs[a] = r < d ? rd[i] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) vs[threadIdx.x + i * NT] = rv[i];
    __syncthreads();
    {
      // 16 lanes per token: squared lengths and k . q
      const int tb = wave * 4 + (lane >> 4), sub = lane & 15;
      float sq = 0.f, sk = 0.f, kq = 0.f;
#pragma unroll
      for (int i = 0; i < RP / 16; ++i) {
        const int a = tb * RPS + lrow<RPT>(sub + 16 * i);
        const float kv = ks[a], qv = qs[a];
        sq += qv * qv;
        sk += kv * kv;
        kq += kv * qv;
      }
      sq = row_sum(sq);
      sk = row_sum(sk);
      kq = row_sum(kq);
      if (sub == 0) {
        const float kn = 1.f / sqrtf(sk + 1e-6f), qn = qscale / sqrtf(sq + 1e-6f);
        *reinterpret_cast<float4*>(sc + 4 * tb) = make_float4(kn, qn, kq * kn * qn, sigmoid_f(rb));
      }
    }
    __syncthreads();
    if (t0 + TB < len) fetch(t0 + TB);
    // lane rg of a column keeps the result of token rg of the block
    float ok[CPL];
#pragma unroll
    for (int c = 0; c < CPL; ++c) ok[c] = 0.f;
    auto read = [&](TokenRegs<RPT, CPL>& x, int tb) {
      const int base = tb * RPS + rg * (RPT + 4);
#pragma unroll
      for (int i = 0; i < RPT; i += 4) {
        ld4(gs + base + i, x.g + i);
        ld4(ks + base + i, x.k + i);
        ld4(qs + base + i, x.q + i);
      }
      ld4(sc + 4 * tb, x.c);
      if constexpr (CPL == 4) {
        ld4(vs + tb * CT + lc, x.v);
      } else {
#pragma unroll
        for (int c = 0; c < CPL; ++c) x.v[c] = vs[tb * CT + lc + c];
      }
    };
    auto step = [&](const TokenRegs<RPT, CPL>& x, int tb) {
      float sk[CPL], sq[CPL];
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        float k0 = 0.f, k1 = 0.f, q0 = 0.f, q1 = 0.f;       // independent chains
#pragma unroll
        for (int i = 0; i < RPT; i += 2) {
          Sr[i][c] *= x.g[i];
          Sr[i + 1][c] *= x.g[i + 1];
          k0 += Sr[i][c] * x.k[i];
          k1 += Sr[i + 1][c] * x.k[i + 1];
          q0 += Sr[i][c] * x.q[i];
          q1 += Sr[i + 1][c] * x.q[i + 1];
        }
        sk[c] = k0 + k1;
        sq[c] = q0 + q1;
      }
      row_sums<CPL>(sk);
#pragma unroll
      for (int c = 0; c < CPL; ++c) sk[c] = x.c[3] * (x.v[c] - x.c[0] * sk[c]);     // u
#pragma unroll
      for (int c = 0; c < CPL; ++c) {
        const float ku = x.c[0] * sk[c];
#pragma unroll
        for (int i = 0; i < RPT; ++i) Sr[i][c] += x.k[i] * ku;
      }
      row_sums<CPL>(sq);
#pragma unroll
      for (int c = 0; c < CPL; ++c) ok[c] = rg == tb ? x.c[1] * sq[c] + x.c[2] * sk[c] : ok[c];
    };
    if (CPL == 1 && nb == TB) {
      // one wave per SIMD: the next token's reads run under the current one's arithmetic
      TokenRegs<RPT, CPL> ra, rb2;
      read(ra, 0);
#pragma unroll 2
      for (int tb = 0; tb < TB; tb += 2) {
        read(rb2, tb + 1);
        step(ra, tb);
        read(ra, (tb + 2) & (TB - 1));
        step(rb2, tb + 1);
      }
    } else {
#pragma unroll 1
      for (int tb = 0; tb < nb; ++tb) {
        TokenRegs<RPT, CPL> ra;
        read(ra, tb);
        step(ra, tb);
      }
    }
    if (rg < nb) {
      float* o = out + (int64_t)(start + t0 + rg) * ow + h * V + col;
#pragma unroll
      for (int c = 0; c < CPL; ++c)
        if (col + c < V) o[c] = ok[c];
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < RPT; ++i)
#pragma unroll
    for (int c = 0; c < CPL; ++c) {
      const int r = rg * RPT + i;
      if (r < d && col + c < V) Sp[(int64_t)r * V + col + c] = Sr[i][c];
    }
}

// One token per row: thread (16 row groups, 16 column lanes of 4 columns); RI: state rows per
// lane (rows rg + 16 i).  V a multiple of 4.
template <typename T, int RI>
__global__ __launch_bounds__(NT) void channel_delta_decode_kernel(
    float* __restrict__ out, const float* __restrict__ qkv, const T* __restrict__ b, int64_t bstr,
    const float* __restrict__ decay, float* __restrict__ S, const int* __restrict__ ctx,
    const int* __restrict__ slots, int row0, int H, int G, int d, int V, int num_slots) {
  __shared__ __align__(16) float kqg[3][16 * RI];
  __shared__ float part[3][NT / 64];
  __shared__ __align__(16) float sums[NT / 64][2][64];
  const int s = blockIdx.x, h = blockIdx.y, g = h / (H / G);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, rg = threadIdx.x >> 4;
  const int cl = (threadIdx.x & 15) * 4, col = blockIdx.z * 64 + cl;
  const bool colok = col < V;
  const int64_t t = row0 + s;
  const int slot = slots[s], pos = ctx[s] - 1;
  float* orow = out + t * H * V + h * V + col;
  if (slot < 0 || slot >= num_slots || pos < 0) {
    if (rg == 0 && colok) *reinterpret_cast<float4*>(orow) = make_float4(0.f, 0.f, 0.f, 0.f);
    return;
  }
  float* Sp = S + ((int64_t)slot * H + h) * d * V + col;
  float4 Sr[RI];
#pragma unroll
  for (int i = 0; i < RI; ++i) {
    const int r = rg + 16 * i;
    Sr[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (pos != 0 && r < d && colok) Sr[i] = *reinterpret_cast<const float4*>(Sp + (int64_t)r * V);
  }
  const float* row = qkv + t * ((int64_t)2 * G * d + (int64_t)H * V);
  float4 v4 = make_float4(0.f, 0.f, 0.f, 0.f);
  if (colok) v4 = *reinterpret_cast<const float4*>(row + 2 * G * d + h * V + col);
  const float bv = to_f(b[t * bstr + h]);
  {
    float kv = 0.f, qv = 0.f;
    const int r = threadIdx.x;
    if (r < 16 * RI) {
      float gv = 0.f;
      if (r < d) {
        kv = row[G * d + g * d + r];
        qv = row[g * d + r];
        gv = decay[t * H * d + h * d + r];
      }
      kqg[0][r] = kv;
      kqg[1][r] = qv;
      kqg[2][r] = gv;
    }
    float a0 = across_rows(row_sum(kv * kv)), a1 = across_rows(row_sum(qv * qv));
    float a2 = across_rows(row_sum(kv * qv));
    if (lane == 0) {
      part[0][wave] = a0;
      part[1][wave] = a1;
      part[2][wave] = a2;
    }
  }
  __syncthreads();
  float ss[3];
#pragma unroll
  for (int j = 0; j < 3; ++j) ss[j] = (part[j][0] + part[j][1]) + (part[j][2] + part[j][3]);
  const float kn = 1.f / sqrtf(ss[0] + 1e-6f), qn = 1.f / sqrtf((float)d) / sqrtf(ss[1] + 1e-6f);
  const float kq = ss[2] * kn * qn, beta = sigmoid_f(bv);
  float sk[4] = {0.f, 0.f, 0.f, 0.f}, sq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < RI; ++i) {
    const int r = rg + 16 * i;
    const float kv = kqg[0][r], qv = kqg[1][r], gv = kqg[2][r];
    Sr[i].x *= gv; Sr[i].y *= gv; Sr[i].z *= gv; Sr[i].w *= gv;
    sk[0] += Sr[i].x * kv; sk[1] += Sr[i].y * kv; sk[2] += Sr[i].z * kv; sk[3] += Sr[i].w * kv;
    sq[0] += Sr[i].x * qv; sq[1] += Sr[i].y * qv; sq[2] += Sr[i].z * qv; sq[3] += Sr[i].w * qv;
  }
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    sk[c] = across_rows(sk[c]);
    sq[c] = across_rows(sq[c]);
  }
  if (lane < 16) {
    *reinterpret_cast<float4*>(&sums[wave][0][cl]) = make_float4(sk[0], sk[1], sk[2], sk[3]);
    *reinterpret_cast<float4*>(&sums[wave][1][cl]) = make_float4(sq[0], sq[1], sq[2], sq[3]);
  }
  __syncthreads();
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    sk[c] = (sums[0][0][cl + c] + sums[1][0][cl + c]) + (sums[2][0][cl + c] + sums[3][0][cl + c]);
    sq[c] = (sums[0][1][cl + c] + sums[1][1][cl + c]) + (sums[2][1][cl + c] + sums[3][1][cl + c]);
  }
  const float u0 = beta * (v4.x - kn * sk[0]), u1 = beta * (v4.y - kn * sk[1]);
  const float u2 = beta * (v4.z - kn * sk[2]), u3 = beta * (v4.w - kn * sk[3]);
  if (!colok) return;
#pragma unroll
  for (int i = 0; i < RI; ++i) {
    const int r = rg + 16 * i;
    if (r < d) {
      const float kv = kn * kqg[0][r];
      *reinterpret_cast<float4*>(Sp + (int64_t)r * V) = make_float4(
          Sr[i].x + kv * u0, Sr[i].y + kv * u1, Sr[i].z + kv * u2, Sr[i].w + kv * u3);
    }
  }
  if (rg == 0)
    *reinterpret_cast<float4*>(orow) = make_float4(qn * sq[0] + kq * u0, qn * sq[1] + kq * u1,
                                                   qn * sq[2] + kq * u2, qn * sq[3] + kq * u3);
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
  const bool mfma = dtype != DT_F32 && ra % 32 == 0 && rg % 32 == 0 && ra <= 256 && rg <= 256 &&
                    ls % 8 == 0 && reinterpret_cast<uintptr_t>(low) % 16 == 0;
  if (mfma) {
    const int nbd = (Nd + 63) / 64, ny = (nbd + (Ng + 63) / 64 + 3) / 4;
    // row tiles per wave: as many as leave a few workgroups per CU
    int tiles = 1;
    while (tiles < 16 && (int64_t)((T_ + 32 * tiles - 1) / (32 * tiles)) * ny >= 1024) tiles <<= 1;
    const dim3 grid((T_ + 16 * tiles - 1) / (16 * tiles), ny);
#define KGC_DG(TT, K)                                                                        \
  delta_gates_mfma_kernel<TT, K><<<grid, NT, 0, s>>>(                                        \
      decay, (TT*)gate, (const TT*)low, ls, (const TT*)a2, (const TT*)g2, neg_a, dt_bias, T_, \
      Nd, Ng, ra, rg, nbd, tiles)
#define KGC_DG_K(TT)                                        \
  do {                                                      \
    const int r = ra > rg ? ra : rg;                        \
    if (r <= 32) KGC_DG(TT, 1);                             \
    else if (r <= 64) KGC_DG(TT, 2);                        \
    else if (r <= 128) KGC_DG(TT, 4);                       \
    else KGC_DG(TT, 8);                                     \
  } while (0)
    if (dtype == DT_BF16) KGC_DG_K(bf16); else KGC_DG_K(f16);
#undef KGC_DG_K
#undef KGC_DG
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
  int rp = 64;
  while (rp < d) rp <<= 1;
  // n sequences: chunks (loc) or single rows from `row0` on
  auto scan = [&](const int* loc, const int* ctx, const int* sl, int n, int row0) {
    if (n <= 0) return;
    // columns per lane: as many as leave two workgroups per CU (256 rows: two at most, for LDS)
    int cpl = rp > 128 ? 2 : 4;
    while (cpl > 1 && (V <= 8 * cpl || (int64_t)n * H * ((V + 16 * cpl - 1) / (16 * cpl)) < 512))
      cpl >>= 1;
    const int ct = 16 * cpl;
    const dim3 grid(n, H, (V + ct - 1) / ct);
    const size_t lds = sizeof(float) * (size_t)(3 * TB * (rp + 64) + TB * ct + TB * 4);
#define KGC_CDS_C(R, C)                                                                      \
  KGC_CD_DISPATCH_T(dtype, channel_delta_scan_kernel<T, R, C><<<grid, NT, lds, s>>>(         \
      out, qkv, (const T*)b, bstr, decay, S, loc, ctx, sl, row0, H, G, d, V, num_slots))
#define KGC_CDS(R)                       \
  do {                                   \
    if (cpl == 4) KGC_CDS_C(R, (R > 8 ? 2 : 4)); \
    else if (cpl == 2) KGC_CDS_C(R, 2);  \
    else KGC_CDS_C(R, 1);                \
  } while (0)
    if (rp == 64) KGC_CDS(4);
    else if (rp == 128) KGC_CDS(8);
    else KGC_CDS(16);
#undef KGC_CDS
#undef KGC_CDS_C
  };
  scan(qsl, seq_lens, slots, P, 0);
  if (D <= 0) return;
  // float4 columns of the state, v and the output
  const bool rows4 = V % 4 == 0 && d % 2 == 0 && reinterpret_cast<uintptr_t>(S) % 16 == 0 &&
                     reinterpret_cast<uintptr_t>(qkv) % 16 == 0 &&
                     reinterpret_cast<uintptr_t>(out) % 16 == 0;
  if (!rows4) {
    scan(nullptr, ctx_lens, slots + P, D, Tp);
    return;
  }
  const dim3 grid(D, H, (V + 63) / 64);
#define KGC_CDD(R)                                                                           \
  KGC_CD_DISPATCH_T(dtype, channel_delta_decode_kernel<T, R><<<grid, NT, 0, s>>>(            \
      out, qkv, (const T*)b, bstr, decay, S, ctx_lens, slots + P, Tp, H, G, d, V, num_slots))
  if (d <= 64) KGC_CDD(4);
  else if (d <= 128) KGC_CDD(8);
  else KGC_CDD(16);
#undef KGC_CDD
}

}  // namespace kgc
