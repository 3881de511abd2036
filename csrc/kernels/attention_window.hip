// Windowed attention with kept first tokens over a plain-layout paged cache
// (k [nb, G, bs, dk], v [nb, G, bs, dv]; dk != dv allowed, any sizes), for the hybrid
// decoders.  Rows are addressed through their strides (krs, vrs elements per cache row), so
// the values may be columns of the key rows (one latent cache row per token).  Query i sees key j when j <= i and (i - j < window or j < keep_first);
// window <= 0 means plain causal attention; ex.chunked: i sees the keys of its own chunk of
// ``window`` positions instead; ex.sink: a score without a value in every softmax.  With pooled blocks (pool > 0) a page holds
// ceil(bs / pool) further rows after its bs token rows: the mean key (value) row of every block
// of pool tokens whose last token lies in the page; query i also sees the blocks that end
// before its window.  Values may be cached turned by their positions (pairs over all dv
// dimensions); a head's output is then turned back by the query's position.
//
//   rope_kv_store     rotates q and k on the first `rot` dims of a head (pair i, i + rot/2,
//                     or 2i, 2i + 1; cos / sin from an fp32 table), writes q, and k / v
//                     into the cache
//   window_attention  one wave per (token, query head): the token's visible keys are the
//                     kept first tokens plus the window, walked 64 keys at a time (one key
//                     per lane for the scores, one value column per lane for P.V) with an
//                     online softmax.  Prefill chunks and decode rows of a step take the
//                     same path, so a position's result does not depend on how the prompt
//                     was cut.  Scores, softmax weights and the weighted sum are fp32.
//   qk_norm_store     RMS norm over the whole q row and the whole k row, rotation of q, k and
//                     v, write of q and into the cache
//   pool_kv           mean rows of the blocks that a step's tokens complete
#include <algorithm>

#include "common.h"
#include "launch.h"

namespace kgc {

namespace {

template <typename T>
__global__ __launch_bounds__(256) void rope_kv_store_kernel(
    const T* __restrict__ qkv, int64_t qkv_stride, const int64_t* __restrict__ positions,
    const float* __restrict__ table, int rot, int table_rows, T* __restrict__ q_out,
    T* __restrict__ k_cache, T* __restrict__ v_cache, const int64_t* __restrict__ slots, int H,
    int G, int dk, int dv, int bs, int num_blocks, bool interleaved) {
  const int64_t t = blockIdx.x;
  const T* row = qkv + t * qkv_stride;
  int64_t pos = positions[t];
  if (pos < 0) pos = 0;
  if (pos >= table_rows) pos = table_rows - 1;        // host checks max_pos; never read past
  const float* cs = table != nullptr ? table + pos * rot : nullptr;
  const int half = rot >> 1;
  const int64_t slot = slots[t];
  const bool store = slot >= 0 && slot < (int64_t)num_blocks * bs;
  const int64_t blk = store ? slot / bs : 0, off = store ? slot % bs : 0;
  // q heads then k heads: (H + G) * dk elements, rotated pairwise on the first `rot` dims
  const int nqk = (H + G) * dk;
  for (int e = threadIdx.x; e < nqk; e += 256) {
    const int head = e / dk, i = e - head * dk;
    float v = to_f(row[e]);
    if (i < rot) {
      // pair p: dims (p, p + rot/2), or (2p, 2p + 1) when interleaved
      const int p = interleaved ? i >> 1 : (i < half ? i : i - half);
      const bool first = interleaved ? !(i & 1) : i < half;
      const int ia = interleaved ? 2 * p : p, ib = interleaved ? 2 * p + 1 : half + p;
      const float c = cs[p], sn = cs[half + p];
      const float a = to_f(row[head * dk + ia]), b = to_f(row[head * dk + ib]);
      float oa, ob;
      neox_rot(a, b, c, sn, oa, ob);
      v = first ? oa : ob;
    }
    if (head < H) {
      q_out[(t * H + head) * dk + i] = from_f<T>(v);
    } else if (store) {
      k_cache[((blk * G + (head - H)) * bs + off) * dk + i] = from_f<T>(v);
    }
  }
  if (store) {
    const T* vrow = row + nqk;
    for (int e = threadIdx.x; e < G * dv; e += 256) {
      const int g = e / dv, i = e - g * dv;
      v_cache[((blk * G + g) * bs + off) * dv + i] = vrow[e];
    }
  }
}

// Attention inputs normed per head: qkv [T, H dk + G dk + G dv] of type TI (row stride qs).
// Each head's q and k (qk_unit) and v (v_unit) is divided by sqrt(mean(x^2) + eps), q and k are
// multiplied by qw / kw [dk] (null: none), q at position p by
// 1 + coef * ln(floor((p + 1) / every) + 1); q goes to q_out [T, H, dk], k and v into the cache.
// fp32 math.  One wave per head vector, any sizes.
template <typename TI, typename T>
__global__ __launch_bounds__(256) void norm_kv_store_kernel(
    const TI* __restrict__ qkv, int64_t qs, const int64_t* __restrict__ positions,
    T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache,
    const int64_t* __restrict__ slots, int H, int G, int dk, int dv, int bs, int num_blocks,
    float eps, bool qk_unit, bool v_unit, float coef, int every, const float* __restrict__ qw,
    const float* __restrict__ kw) {
  const int64_t t = blockIdx.x;
  const TI* row = qkv + t * qs;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  int64_t pos = positions[t];
  if (pos < 0) pos = 0;
  const float temp = coef != 0.f ? 1.f + coef * logf((float)((pos + 1) / every) + 1.f) : 1.f;
  const int64_t slot = slots[t];
  const bool store = slot >= 0 && slot < (int64_t)num_blocks * bs;
  const int64_t blk = store ? slot / bs : 0, off = store ? slot % bs : 0;
  for (int hv = wave; hv < H + 2 * G; hv += 4) {
    const bool isq = hv < H, isk = !isq && hv < H + G;
    const int n = hv < H + G ? dk : dv;
    const TI* src = row + (hv < H + G ? hv * dk : (H + G) * dk + (hv - H - G) * dv);
    if (!isq && !store) continue;
    float f = isq ? temp : 1.f;
    if (isq || isk ? qk_unit : v_unit) {
      float ss = 0.f;
      for (int i = lane; i < n; i += 64) {
        const float v = to_f(src[i]);
        ss += v * v;
      }
      ss = wave_sum(ss);
      f /= sqrtf(ss / (float)n + eps);
    }
    const float* w = isq ? qw : isk ? kw : nullptr;
    T* dst = isq ? q_out + (t * H + hv) * dk
                 : isk ? k_cache + ((blk * G + (hv - H)) * bs + off) * dk
                       : v_cache + ((blk * G + (hv - H - G)) * bs + off) * dv;
    for (int i = lane; i < n; i += 64)
      dst[i] = from_f<T>(to_f(src[i]) * f * (w != nullptr ? w[i] : 1.f));
  }
}

// first position that a query at `pos` sees
__device__ __forceinline__ int first_visible(int pos, int window, bool chunked) {
  if (window <= 0) return 0;
  return chunked ? pos - pos % window : max(0, pos - window + 1);
}

// whole blocks of `pool` tokens that end before the window of a query at `pos`
__device__ __forceinline__ int pooled_count(int pos, int window, int pool) {
  const int n = pos - window + 1;
  return n > 0 ? n / pool : 0;
}

// pooled block b lives in the page of its last token, after the page's token rows
__device__ __forceinline__ void pooled_place(int b, int pool, int bs, int& page, int& row) {
  page = (b * pool + pool - 1) / bs;
  row = bs + b - page * bs / pool;
}

// The mean row of the block that ends at token `pos`, for kv head g: threads tid, tid + nthr,
// ... take one column each (keys, then values).
template <typename T>
__device__ __forceinline__ void pool_block(T* k_cache, T* v_cache, const int* bt, int pos,
                                           int pool, int g, int G, int dk, int dv, int krs,
                                           int vrs, int bs, int prow, int num_blocks, int tid,
                                           int nthr) {
  int pg, pr;
  pooled_place(pos / pool, pool, bs, pg, pr);
  int db = bt[pg];
  if (db < 0 || db >= num_blocks) db = 0;
  const int64_t dst = (int64_t)(db * G + g) * prow + pr;
  const float inv = 1.f / (float)pool;
  for (int c = tid; c < dk + dv; c += nthr) {
    T* base = c < dk ? k_cache + c : v_cache + (c - dk);
    const int rs = c < dk ? krs : vrs;
    float a = 0.f;
#pragma unroll 8
    for (int j = pos + 1 - pool; j <= pos; ++j) {
      int b = bt[j / bs];
      if (b < 0 || b >= num_blocks) b = 0;
      a += to_f(base[((int64_t)(b * G + g) * prow + j % bs) * rs]);
    }
    base[dst * rs] = from_f<T>(a * inv);
  }
}

// the table row of a position (never past the table)
__device__ __forceinline__ const float* rot_row(const WindowExtra& ex, int pos, int dv) {
  return ex.vtab + (int64_t)min(pos, ex.vrows - 1) * dv;
}

// column c of a head's output turned back by the row's position: `self` and `other` are the
// pair's members, cs the table row (cos | sin)
__device__ __forceinline__ float turn_back(float self, float other, const float* cs, int c,
                                           int dv, bool inter) {
  const int half = dv >> 1;
  const int m = inter ? c >> 1 : (c < half ? c : c - half);
  const bool first = inter ? !(c & 1) : c < half;
  const float cn = cs[m], sn = cs[half + m];
  return first ? self * cn + other * sn : self * cn - other * sn;
}
__device__ __forceinline__ int turn_partner(int c, int dv, bool inter) {
  return inter ? c ^ 1 : (c < (dv >> 1) ? c + (dv >> 1) : c - (dv >> 1));
}

constexpr int MAX_DV_PER_LANE = 16;    // dv <= 1024

// scaled score -> cap * tanh(score / cap) when a cap is set
__device__ __forceinline__ float cap_score(float s, float cap) {
  return cap > 0.f ? cap * tanhf(s / cap) : s;
}

// sigmoid of the element-wise output gate at (row t, column c of the concatenated heads)
template <typename T>
__device__ __forceinline__ float elem_gate(const WindowExtra& ex, int64_t t, int c) {
  if (ex.egate == nullptr) return 1.f;
  const float g = to_f(static_cast<const T*>(ex.egate)[t * ex.egs + c]);
  return 1.f / (1.f + expf(-g));
}

// grid (T, H), one wave.  LDS: q row [dk] fp32, p [64], value-row offsets [64], and with
// rotated values the output row [dv].
template <typename T>
__global__ __launch_bounds__(64) void window_attention_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ k_cache,
    const T* __restrict__ v_cache, const int* __restrict__ qsl, const int* __restrict__ seq_lens,
    const int* __restrict__ pbt, const int* __restrict__ ctx_lens, const int* __restrict__ dbt,
    int bt_stride, int P, int Tp, int H, int G, int dk, int dv, int krs, int vrs, int bs,
    int num_blocks, float scale, int window, int keep_first, const float* __restrict__ gate, int kinds,
    WindowExtra ex) {
  extern __shared__ float lds[];
  if (!(kinds & (blockIdx.x < Tp ? 1 : 2))) return;   // rows another kernel of the step owns
  float* qs = lds;                  // [dk]
  float* pw = lds + dk;             // [64]
  int* voff = (int*)(pw + 64);      // [64] (block * G + g) * bs + row
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int g = h / (H / G);
  T* orow = out + (int64_t)t * ex.ors + h * dv;
  int pos;
  const int* bt;
  if (t < Tp) {
    int lo = 0, hi = P - 1;          // the sequence whose rows [qsl[i], qsl[i+1]) hold t
    while (lo < hi) {
      const int mid = (lo + hi + 1) >> 1;
      if (qsl[mid] <= t) lo = mid; else hi = mid - 1;
    }
    pos = seq_lens[lo] - (qsl[lo + 1] - qsl[lo]) + (t - qsl[lo]);
    bt = pbt + (int64_t)lo * bt_stride;
  } else {
    const int dd = t - Tp;
    pos = ctx_lens[dd] - 1;
    bt = dbt + (int64_t)dd * bt_stride;
  }
  if (pos < 0 || pos >= bt_stride * bs) {      // a padding row (or nothing to attend)
    for (int c = lane; c < dv; c += 64) orow[c] = from_f<T>(0.f);
    return;
  }
  const T* qrow = q + ((int64_t)t * H + h) * dk;
  for (int c = lane; c < dk; c += 64) qs[c] = to_f(qrow[c]);
  __syncthreads();
  const int lo_w = first_visible(pos, window, ex.chunked);
  // kept first tokens outside the window, or the pooled blocks before it
  const int ns = ex.pool > 0 ? pooled_count(pos, window, ex.pool) : min(keep_first, lo_w);
  const int total = ns + (pos - lo_w + 1);
  float m = ex.sink, l = ex.sink > -INFINITY ? 1.f : 0.f;
  float acc[MAX_DV_PER_LANE];
#pragma unroll
  for (int u = 0; u < MAX_DV_PER_LANE; ++u) acc[u] = 0.f;
  for (int base = 0; base < total; base += 64) {
    const int idx = base + lane;
    const bool ok = idx < total;
    float s = -INFINITY;
    int ro = 0;
    if (ok) {
      const int j = idx < ns ? idx : lo_w + (idx - ns);
      int pg = j / bs, pr = j % bs;
      if (ex.pool > 0 && idx < ns) pooled_place(idx, ex.pool, bs, pg, pr);
      int b = bt[pg];
      if (b < 0 || b >= num_blocks) b = 0;       // never index outside the pool
      ro = (b * G + g) * ex.prow + pr;
      const T* kr = k_cache + (int64_t)ro * krs;
      float d = 0.f;
      for (int c = 0; c < dk; ++c) d += qs[c] * to_f(kr[c]);
      s = cap_score(d * scale, ex.softcap);
    }
    const float mn = fmaxf(m, wave_max(s));
    const float alpha = expf(m - mn);             // m = -inf at first: exp(-inf) = 0
    const float p = ok ? expf(s - mn) : 0.f;
    l = l * alpha + wave_sum(p);
    m = mn;
    __syncthreads();                              // the previous chunk's pw / voff were read
    pw[lane] = p;
    voff[lane] = ro;
    __syncthreads();
    const int cnt = min(64, total - base);
#pragma unroll
    for (int u = 0; u < MAX_DV_PER_LANE; ++u) {
      const int c = lane + 64 * u;
      if (c < dv) {
        float a = acc[u] * alpha;
        for (int jj = 0; jj < cnt; ++jj) a += pw[jj] * to_f(v_cache[(int64_t)voff[jj] * vrs + c]);
        acc[u] = a;
      }
    }
  }
  const float gt = (gate != nullptr ? gate[(int64_t)t * H + h] : 1.f) * ex.out_scale;
  const float inv = gt / l;
  if (ex.vtab != nullptr) {
    float* os = (float*)(voff + 64);              // [dv]
#pragma unroll
    for (int u = 0; u < MAX_DV_PER_LANE; ++u)
      if (lane + 64 * u < dv) os[lane + 64 * u] = acc[u];
    __syncthreads();
    const float* cs = rot_row(ex, pos, dv);
#pragma unroll
    for (int u = 0; u < MAX_DV_PER_LANE; ++u) {
      const int c = lane + 64 * u;
      if (c < dv)
        acc[u] = turn_back(acc[u], os[turn_partner(c, dv, ex.vinter)], cs, c, dv, ex.vinter);
    }
  }
#pragma unroll
  for (int u = 0; u < MAX_DV_PER_LANE; ++u) {
    const int c = lane + 64 * u;
    if (c < dv) orow[c] = from_f<T>(acc[u] * inv * elem_gate<T>(ex, t, h * dv + c));
  }
}

// ---- 8 consecutive elements of a cache row as fp32 (16-byte loads; dk % 8 == 0)
template <typename T>
__device__ __forceinline__ void load8(const T* p, float (&v)[8]) {
  if constexpr (std::is_same_v<T, float>) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    const float4 b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
    v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
  } else {
    Pack8<T> t;
    t.u = *reinterpret_cast<const u32x4*>(p);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = to_f(t.h[e]);
  }
}

// the same 8 elements kept as loaded (4 registers for 16-bit types) until they are used
template <typename T> struct Raw8 { u32x4 u; };
template <> struct Raw8<float> { float4 a, b; };

template <typename T>
__device__ __forceinline__ Raw8<T> load8raw(const T* p) {
  Raw8<T> r;
  if constexpr (std::is_same_v<T, float>) {
    r.a = *reinterpret_cast<const float4*>(p);
    r.b = *reinterpret_cast<const float4*>(p + 4);
  } else {
    r.u = *reinterpret_cast<const u32x4*>(p);
  }
  return r;
}

template <typename T>
__device__ __forceinline__ void cvt8(const Raw8<T>& r, float (&v)[8]) {
  if constexpr (std::is_same_v<T, float>) {
    v[0] = r.a.x; v[1] = r.a.y; v[2] = r.a.z; v[3] = r.a.w;
    v[4] = r.b.x; v[5] = r.b.y; v[6] = r.b.z; v[7] = r.b.w;
  } else {
    Pack8<T> t;
    t.u = r.u;
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = to_f(t.h[e]);
  }
}

template <typename T>
__device__ __forceinline__ void load2(const T* p, float& a, float& b) {
  if constexpr (std::is_same_v<T, float>) {
    const float2 t = *reinterpret_cast<const float2*>(p);
    a = t.x;
    b = t.y;
  } else {
    union { uint32_t u; T h[2]; } t;
    t.u = *reinterpret_cast<const uint32_t*>(p);
    a = to_f(t.h[0]);
    b = to_f(t.h[1]);
  }
}

// Decode rows: one workgroup of 8 waves per (row, kv head, group of up to QH query heads).
// The visible keys (kept first tokens + window) are cut into 64-key chunks dealt round-robin
// to the waves.  In a chunk each lane takes one key: its row is read once (16-byte loads)
// and dotted with every query head of the group (q in LDS as fp32); then each lane takes
// two value columns and walks the chunk's 64 value rows, again once for all heads.  Every
// wave carries its own online-softmax state per head; the eight states merge in LDS in
// wave order (deterministic).  Scores, weights and sums are fp32.
constexpr int DEC_WAVES = 8;          // waves per workgroup (4 when the grid is large)
constexpr int DEC_UMAX = 4;          // value columns per lane: 2 * DEC_UMAX * 64 >= dv

// EXT: pooled blocks and rotated values (the caches are not __restrict__ there: the workgroup
// of a kv head's first query heads also writes the mean row of a block its row completes,
// which no row of the step sees yet).
template <typename T, int QH, int NWV, bool EXT>
__global__ __launch_bounds__(64 * NWV) void window_decode_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* k_cache, const T* v_cache, const int* __restrict__ ctx_lens, const int* __restrict__ dbt,
    int bt_stride, int Tp, int H, int G, int dk, int dv, int krs, int vrs, int bs, int num_blocks,
    float scale, int window, int keep_first, const float* __restrict__ gate, WindowExtra ex) {
  extern __shared__ float lds[];
  const int dd = blockIdx.x, g = blockIdx.y, qpg = H / G, hq0 = blockIdx.z * QH;
  const int nh = min(QH, qpg - hq0);
  const int t = Tp + dd, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  float* qs = lds;                                    // [QH][dk]
  float* pb = qs + QH * dk;                           // [waves][QH][64]
  int* ob = (int*)(pb + NWV * QH * 64);         // [waves][64]
  float* mm = (float*)(ob + NWV * 64);          // [waves][QH]
  float* ml = mm + NWV * QH;                    // [waves][QH]
  float* accs = ml + NWV * QH;                  // [QH][dv]
  const int h0 = g * qpg + hq0;                       // first query head of this workgroup
  const int pos = ctx_lens[dd] - 1;
  const int* bt = dbt + (int64_t)dd * bt_stride;
  if (pos < 0 || pos >= bt_stride * bs) {             // a padding row: zeros
    for (int e = threadIdx.x; e < nh * dv; e += 64 * NWV)
      out[(int64_t)t * ex.ors + h0 * dv + e] = from_f<T>(0.f);
    return;
  }
  for (int e = threadIdx.x; e < nh * dk; e += 64 * NWV)
    qs[e] = to_f(q[((int64_t)t * H + h0) * dk + e]);
  for (int e = threadIdx.x; e < QH * dv; e += 64 * NWV) accs[e] = 0.f;
  __syncthreads();
  const int lo_w = first_visible(pos, window, ex.chunked);
  int ns = min(keep_first, lo_w);
  if constexpr (EXT) {
    if (ex.pool > 0) {
      ns = pooled_count(pos, window, ex.pool);
      if (blockIdx.z == 0 && (pos + 1) % ex.pool == 0)
        pool_block<T>(const_cast<T*>(k_cache), const_cast<T*>(v_cache), bt, pos, ex.pool, g, G, dk,
                      dv, krs, vrs, bs, ex.prow, num_blocks, threadIdx.x, 64 * NWV);
    }
  }
  const int total = ns + (pos - lo_w + 1);
  const int nchunks = (total + 63) >> 6;
  float m[QH], l[QH], acc[QH][DEC_UMAX][2];
#pragma unroll
  for (int h = 0; h < QH; ++h) {
    m[h] = wave == 0 ? ex.sink : -INFINITY;           // (the first wave always has keys)
    l[h] = m[h] > -INFINITY ? 1.f : 0.f;
#pragma unroll
    for (int u = 0; u < DEC_UMAX; ++u) acc[h][u][0] = acc[h][u][1] = 0.f;
  }
  float* pw = pb + wave * QH * 64;
  int* ow = ob + wave * 64;
  const int lpr = dv >> 3;                 // lanes per value row in the 16-byte path
  const bool vrow = (dv & 7) == 0 && lpr >= 1 && lpr <= 64;
  const bool vpow2 = (lpr & (lpr - 1)) == 0;
  const int kg = vrow ? 64 / lpr : 1;      // lane groups (lanes past kg * lpr idle)
  for (int chunk = wave; chunk < nchunks; chunk += NWV) {
    const int idx = chunk * 64 + lane;
    const bool ok = idx < total;
    float sc[QH];
#pragma unroll
    for (int h = 0; h < QH; ++h) sc[h] = 0.f;
    int ro = 0;
    if (ok) {
      const int j = idx < ns ? idx : lo_w + (idx - ns);
      int pg = j / bs, pr = j % bs;
      if constexpr (EXT) {
        if (ex.pool > 0 && idx < ns) pooled_place(idx, ex.pool, bs, pg, pr);
      }
      int b = bt[pg];
      if (b < 0 || b >= num_blocks) b = 0;
      ro = (b * G + g) * (EXT ? ex.prow : bs) + pr;
      const T* kr = k_cache + (int64_t)ro * krs;
      constexpr int KB = 8;                       // 16-byte pieces of the key row in flight
      for (int c0 = 0; c0 < dk; c0 += 8 * KB) {
        Raw8<T> kraw[KB];
#pragma unroll
        for (int b = 0; b < KB; ++b) {
          const int c = min(c0 + 8 * b, dk - 8);  // clamped: pieces past dk are not used
          kraw[b] = load8raw(kr + c);
        }
#pragma unroll
        for (int b = 0; b < KB; ++b) {
          const int c = c0 + 8 * b;
          if (c < dk) {
            float kv[8];
            cvt8(kraw[b], kv);
#pragma unroll
            for (int h = 0; h < QH; ++h) {
              if (h < nh) {
                const float* qh = qs + h * dk + c;
#pragma unroll
                for (int e = 0; e < 8; ++e) sc[h] += qh[e] * kv[e];
              }
            }
          }
        }
      }
    }
    float alpha[QH];
#pragma unroll
    for (int h = 0; h < QH; ++h) {
      const float sv = ok ? cap_score(sc[h] * scale, ex.softcap) : -INFINITY;
      const float mn = fmaxf(m[h], wave_max(sv));
      alpha[h] = expf(m[h] - mn);
      const float p = ok ? expf(sv - mn) : 0.f;
      l[h] = l[h] * alpha[h] + wave_sum(p);
      m[h] = mn;
      pw[h * 64 + lane] = p;
    }
    ow[lane] = ro;
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    const int cnt = min(64, total - chunk * 64);
    if (vrow) {
      // lpr lanes cover a value row with 16-byte loads; the 64 / lpr lane groups take
      // every (64 / lpr)-th key of the chunk and are summed once, after the last chunk
#pragma unroll
      for (int h = 0; h < QH; ++h)
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[h][e >> 1][e & 1] *= alpha[h];
      const int cg = lane / lpr, ci = lane - cg * lpr;
      constexpr int VB = std::is_same_v<T, float> ? 4 : 8;    // rows in flight per lane
      for (int j0 = cg < kg ? cg : cnt; j0 < cnt; j0 += VB * kg) {
        Raw8<T> raw[VB];
#pragma unroll
        for (int b = 0; b < VB; ++b) {
          const int jj = min(j0 + b * kg, cnt - 1);            // clamped: weight 0 below
          raw[b] = load8raw(v_cache + (int64_t)ow[jj] * vrs + 8 * ci);
        }
#pragma unroll
        for (int b = 0; b < VB; ++b) {
          const int jj = j0 + b * kg;
          float v8[8];
          cvt8(raw[b], v8);
#pragma unroll
          for (int h = 0; h < QH; ++h) {
            const float p = jj < cnt ? pw[h * 64 + min(jj, 63)] : 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[h][e >> 1][e & 1] += p * v8[e];
          }
        }
      }
    } else {
#pragma unroll
    for (int u = 0; u < DEC_UMAX; ++u) {
      const int c0 = 2 * lane + 128 * u;
      if (c0 < dv) {
        float a0[QH], a1[QH];
#pragma unroll
        for (int h = 0; h < QH; ++h) {
          a0[h] = acc[h][u][0] * alpha[h];
          a1[h] = acc[h][u][1] * alpha[h];
        }
        for (int jj = 0; jj < cnt; ++jj) {
          float v0, v1;
          load2(v_cache + (int64_t)ow[jj] * vrs + c0, v0, v1);
#pragma unroll
          for (int h = 0; h < QH; ++h) {
            const float p = pw[h * 64 + jj];
            a0[h] += p * v0;
            a1[h] += p * v1;
          }
        }
#pragma unroll
        for (int h = 0; h < QH; ++h) {
          acc[h][u][0] = a0[h];
          acc[h][u][1] = a1[h];
        }
      }
    }
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  if (lane == 0) {
#pragma unroll
    for (int h = 0; h < QH; ++h) {
      mm[wave * QH + h] = m[h];
      ml[wave * QH + h] = l[h];
    }
  }
  __syncthreads();
  float f[QH];
#pragma unroll
  for (int h = 0; h < QH; ++h) {
    float M = -INFINITY;
    for (int w = 0; w < NWV; ++w) M = fmaxf(M, mm[w * QH + h]);
    f[h] = m[h] == -INFINITY ? 0.f : expf(m[h] - M);
  }
  if (vrow && vpow2) {
    for (int off = lpr; off < 64; off <<= 1)
#pragma unroll
      for (int h = 0; h < QH; ++h)
#pragma unroll
        for (int e = 0; e < 8; ++e)
          acc[h][e >> 1][e & 1] += __shfl_xor(acc[h][e >> 1][e & 1], off, 64);
  } else if (vrow) {
    // lane groups of any width: the first group gathers the others' sums (lanes past it
    // read wrapped lanes; their sums are not used)
#pragma unroll
    for (int h = 0; h < QH; ++h)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float own = acc[h][e >> 1][e & 1];
        float tot = own;
        for (int g2 = 1; g2 < kg; ++g2) tot += __shfl(own, (lane + g2 * lpr) & 63, 64);
        acc[h][e >> 1][e & 1] = tot;
      }
  }
  for (int w = 0; w < NWV; ++w) {
    if (vrow) {
      if (wave == w && nchunks > w && lane < lpr) {
#pragma unroll
        for (int h = 0; h < QH; ++h)
#pragma unroll
          for (int e = 0; e < 8; ++e) accs[h * dv + 8 * lane + e] += acc[h][e >> 1][e & 1] * f[h];
      }
    } else if (wave == w && nchunks > w) {
#pragma unroll
      for (int u = 0; u < DEC_UMAX; ++u) {
        const int c0 = 2 * lane + 128 * u;
        if (c0 < dv) {
#pragma unroll
          for (int h = 0; h < QH; ++h) {
            accs[h * dv + c0] += acc[h][u][0] * f[h];
            accs[h * dv + c0 + 1] += acc[h][u][1] * f[h];
          }
        }
      }
    }
    __syncthreads();
  }
  for (int e = threadIdx.x; e < nh * dv; e += 64 * NWV) {
    const int h = e / dv;
    float M = -INFINITY, L = 0.f;
    for (int w = 0; w < NWV; ++w) M = fmaxf(M, mm[w * QH + h]);
    for (int w = 0; w < NWV; ++w) {
      const float mw = mm[w * QH + h];
      if (mw != -INFINITY) L += ml[w * QH + h] * expf(mw - M);
    }
    const float gt = (gate != nullptr ? gate[(int64_t)t * H + h0 + h] : 1.f) * ex.out_scale;
    float a = accs[e];
    if constexpr (EXT) {
      if (ex.vtab != nullptr) {
        const int c = e - h * dv;
        a = turn_back(a, accs[h * dv + turn_partner(c, dv, ex.vinter)], rot_row(ex, pos, dv), c,
                      dv, ex.vinter);
      }
    }
    out[(int64_t)t * ex.ors + h0 * dv + e] =
        from_f<T>(a * gt / L * elem_gate<T>(ex, t, h0 * dv + e));
  }
}

// Decode rows on the matrix cores (16-bit activations): one workgroup of NWV waves per (row, kv
// head, group of up to 16 query heads).  The visible keys are cut into 32-key chunks dealt
// round-robin to the waves.  Per chunk and wave, with the heads as columns (lane & 15):
//   S^T = K . Q^T   two 16-key tiles, A fragments straight from the cache rows (A row m is key
//                   8 (m >> 2) + (m & 3), + 4 in the second tile),
//   online softmax in fp32, statistics per head in the lane,
//   O^T += V^T . P^T with P^T straight from the S^T accumulators as a pair of values (value +
//                   remainder) and V^T through the wave's own piece of LDS; where the values are
//                   columns of the key rows the key fragments are what is written there.
// The waves' states meet in LDS at the end, in wave order.
constexpr int DM_VST = 40;             // elements per V^T row: 32 keys + 8

template <typename T, int KS, int DT, int NWV>
__global__ __launch_bounds__(64 * NWV) void window_decode_mfma_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ k_cache,
    const T* __restrict__ v_cache, const int* __restrict__ ctx_lens, const int* __restrict__ dbt,
    int bt_stride, int Tp, int H, int G, int dk, int dv, int krs, int vrs, int bs, int num_blocks,
    float scale, int window, int keep_first, const float* __restrict__ gate, bool shared,
    WindowExtra ex) {
  typedef typename Vec8<T>::type V8;
  constexpr int VBYTES = NWV * DT * 16 * DM_VST * 2, OBYTES = NWV * 16 * DT * 16 * 4;
  __shared__ __attribute__((aligned(16))) char smem[VBYTES > OBYTES ? VBYTES : OBYTES];
  __shared__ float mm[NWV][16], ml[NWV][16];
  const int dd = blockIdx.x, g = blockIdx.y, qpg = H / G, hq0 = blockIdx.z * 16;
  const int nh = min(16, qpg - hq0), h0 = g * qpg + hq0, t = Tp + dd;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, qd = lane >> 4;
  const int pos = ctx_lens[dd] - 1;
  const int* bt = dbt + (int64_t)dd * bt_stride;
  if (pos < 0 || pos >= bt_stride * bs) {             // a padding row: zeros
    for (int e = threadIdx.x; e < nh * dv; e += 64 * NWV)
      out[(int64_t)t * ex.ors + h0 * dv + e] = from_f<T>(0.f);
    return;
  }
  V8 qf[KS];
  {
    const T* qrow = q + ((int64_t)t * H + h0 + min(r16, nh - 1)) * dk;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      Pack8<T> p;
      p.u = u32x4{0u, 0u, 0u, 0u};
      if (32 * s + 8 * qd < dk) p.u = *reinterpret_cast<const u32x4*>(qrow + 32 * s + 8 * qd);
      qf[s] = p.v;
    }
  }
  const int lo_w = first_visible(pos, window, ex.chunked), ns = min(keep_first, lo_w);
  const int total = ns + (pos - lo_w + 1), nch = (total + 31) >> 5;
  const int keyA = 8 * (r16 >> 2) + (r16 & 3);
  T* vt = reinterpret_cast<T*>(smem) + wave * DT * 16 * DM_VST;
  float m = wave == 0 ? ex.sink : -INFINITY;          // (the first wave always has keys)
  float l = qd == 0 && m > -INFINITY ? 1.f : 0.f;
  f32x4 o[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int ch = wave; ch < nch; ch += NWV) {
    Pack8<T> kf[2][KS];
    int64_t row[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int idx = min(32 * ch + keyA + 4 * j, total - 1);      // clamped: weight 0 below
      const int key = idx < ns ? idx : lo_w + (idx - ns);
      int b = bt[key / bs];
      if (b < 0 || b >= num_blocks) b = 0;
      row[j] = (int64_t)(b * G + g) * bs + key % bs;
      const T* kr = k_cache + row[j] * krs + 8 * qd;
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        kf[j][s].u = u32x4{0u, 0u, 0u, 0u};
        if (32 * s + 8 * qd < dk) kf[j][s].u = *reinterpret_cast<const u32x4*>(kr + 32 * s);
      }
    }
    Pack8<T> vf[2][DT / 2];
    if (!shared) {
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const T* vr = v_cache + row[j] * vrs + 8 * qd;
#pragma unroll
        for (int s = 0; s < DT / 2; ++s) {
          vf[j][s].u = u32x4{0u, 0u, 0u, 0u};
          if (32 * s + 8 * qd < dv) vf[j][s].u = *reinterpret_cast<const u32x4*>(vr + 32 * s);
        }
      }
    }
    f32x4 sc[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      f32x4 a = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) a = mfma16x16x32(kf[j][s].v, qf[s], a);
      sc[j] = a;
    }
    // V^T of the chunk, while the products are under way
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");    // (the last chunk's fragments were read)
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int s = 0; s < DT / 2; ++s) {
      if (32 * s + 8 * qd < dv) {
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
          for (int e = 0; e < 8; ++e)
            vt[(32 * s + 8 * qd + e) * DM_VST + keyA + 4 * j] =
                shared ? kf[j][s < KS ? s : 0].h[e] : vf[j][s].h[e];
      }
    }
    float tmax = -INFINITY;
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool ok = 32 * ch + 8 * qd + 4 * j + i < total;
        sc[j][i] = ok ? cap_score(sc[j][i] * scale, ex.softcap) : -INFINITY;
        tmax = fmaxf(tmax, sc[j][i]);
      }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float mn = fmaxf(m, tmax);
    const float alpha = m == -INFINITY ? 0.f : __expf(m - mn);
    m = mn;
    l *= alpha;
    Pack8<T> ph, pl;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float pa = sc[0][i] == -INFINITY ? 0.f : __expf(sc[0][i] - mn);
      const float pb = sc[1][i] == -INFINITY ? 0.f : __expf(sc[1][i] - mn);
      l += pa + pb;
      ph.h[i] = from_f<T>(pa);
      ph.h[4 + i] = from_f<T>(pb);
      pl.h[i] = from_f<T>(pa - to_f(ph.h[i]));
      pl.h[4 + i] = from_f<T>(pb - to_f(ph.h[4 + i]));
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int d = 0; d < DT; ++d) {
      if (16 * d < dv) {
        Pack8<T> fr;
        fr.u = *reinterpret_cast<const u32x4*>(vt + (16 * d + r16) * DM_VST + 8 * qd);
        f32x4 a = o[d] * alpha;
        a = mfma16x16x32(fr.v, ph.v, a);
        o[d] = mfma16x16x32(fr.v, pl.v, a);
      }
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (qd == 0) {
    mm[wave][r16] = m;
    ml[wave][r16] = l;
  }
  __syncthreads();
  float M = -INFINITY;
#pragma unroll
  for (int w = 0; w < NWV; ++w) M = fmaxf(M, mm[w][r16]);
  const float f = m == -INFINITY ? 0.f : __expf(m - M);
  float* ob = reinterpret_cast<float*>(smem);         // [NWV][16][DT * 16]
#pragma unroll
  for (int d = 0; d < DT; ++d)
    *reinterpret_cast<f32x4*>(ob + (wave * 16 + r16) * DT * 16 + 16 * d + 4 * qd) = o[d] * f;
  __syncthreads();
  for (int e = threadIdx.x; e < nh * dv; e += 64 * NWV) {
    const int h = e / dv, c = e - h * dv;
    float Mh = -INFINITY, L = 0.f, a = 0.f;
#pragma unroll
    for (int w = 0; w < NWV; ++w) Mh = fmaxf(Mh, mm[w][h]);
#pragma unroll
    for (int w = 0; w < NWV; ++w) {
      const float mw = mm[w][h];
      if (mw != -INFINITY) L += ml[w][h] * __expf(mw - Mh);
      a += ob[(w * 16 + h) * DT * 16 + c];
    }
    const float gt = (gate != nullptr ? gate[(int64_t)t * H + h0 + h] : 1.f) * ex.out_scale;
    out[(int64_t)t * ex.ors + h0 * dv + e] =
        from_f<T>(a * gt / L * elem_gate<T>(ex, t, h0 * dv + e));
  }
}

// Prefill chunks on the matrix cores (16-bit activations).  One workgroup of 4 waves per
// (64 query rows of a chunk, query head); wave w owns rows 16 w .. 16 w + 15.  Keys come in
// 64-key tiles -- first the kept first tokens that lie before the tile's earliest window,
// then the span from that window's start to the last row -- gathered from the pages into
// LDS as K [64][dk, padded to 32, + 8] and V^T [dv][64 + 8].  Per tile and wave:
//   S^T = K . Q^T   (v_mfma_f32_16x16x32; the query is lane & 15 in every accumulator, so
//                    the softmax statistics are lane-local up to two shuffles),
//   visibility mask, online softmax in fp32,
//   O^T += V^T . P^T with P^T taken straight from the S^T accumulators (key m of an A row
//                    is 8 (m >> 2) + (m & 3), + 4 for the second tile of a 32-key pair).
// The fp32 weights enter that product as a bf16/f16 pair (value + remainder), two MFMAs,
// so they carry ~16 mantissa bits rather than 8.
// EXT: tiles of pooled blocks take the place of the kept first tokens, and with values rotated
// in halves the rows of V^T alternate 16 columns of the first half and 16 of the second, so
// that both members of a pair sit in one lane's accumulators and are turned back in registers.
constexpr int PFW_BM = 64, PFW_BN = 64, PFW_KPAD = 8, PFW_VPAD = 8;

template <typename T, int KSM, int DTM, bool EXT>
__global__ __launch_bounds__(256, KSM <= 4 ? 3 : 2) void window_prefill_mfma_kernel(
    T* __restrict__ out, const T* __restrict__ q, const T* __restrict__ k_cache,
    const T* __restrict__ v_cache, const int* __restrict__ qsl, const int* __restrict__ seq_lens,
    const int* __restrict__ pbt, int bt_stride, const int* __restrict__ work_seq,
    const int* __restrict__ work_blk, int blk_rows, int H, int G, int dk, int dv, int krs,
    int vrs, int bs, int num_blocks, float scale, int window, int keep_first, const float* __restrict__ gate,
    WindowExtra ex) {
  typedef typename Vec8<T>::type V8;
  extern __shared__ float lds_f[];
  T* Ks = reinterpret_cast<T*>(lds_f);                 // [64][kp + 8]
  const int kp = (dk + 31) & ~31;                      // key rows padded with zeros in LDS
  const int kst = kp + PFW_KPAD, vst = PFW_BN + PFW_VPAD;
  T* Vt = Ks + PFW_BN * kst;                           // [dv][64 + 8]
  // heads run fastest: workgroups are dealt round-robin over the XCDs, so every XCD sees all row
  // blocks of its heads (with chunks the cost of a block depends on its place)
  const int item = blockIdx.y / (blk_rows / PFW_BM), sub = blockIdx.y % (blk_rows / PFW_BM);
  const int seq = work_seq[item], h = blockIdx.x, g = h / (H / G);
  const int q0 = qsl[seq], qlen = qsl[seq + 1] - q0, ctx0 = seq_lens[seq] - qlen;
  const int r0 = work_blk[item] * blk_rows + sub * PFW_BM;
  if (r0 >= qlen || ctx0 < 0) return;
  const int rows = min(PFW_BM, qlen - r0);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, qd = lane >> 4;
  const int nks = kp >> 5, ndt = dv >> 4;
  const int* bt = pbt + (int64_t)seq * bt_stride;
  const int myrow = r0 + 16 * wave + r16;
  const bool rowok = myrow < qlen;
  const int qpos = ctx0 + myrow;
  // this wave's q fragments: lane (r16, qd) holds dims 32 s + 8 qd .. + 7 of its row
  V8 qf[KSM];
  {
    const T* qrow = q + ((int64_t)(q0 + (rowok ? myrow : r0)) * H + h) * dk;
#pragma unroll
    for (int s2 = 0; s2 < KSM; ++s2) {
      Pack8<T> tq;
      tq.u = u32x4{0u, 0u, 0u, 0u};
      if (32 * s2 + 8 * qd < dk && rowok) tq.u = *reinterpret_cast<const u32x4*>(qrow + 32 * s2 + 8 * qd);
      qf[s2] = tq.v;
    }
  }
  f32x4 o[DTM];
#pragma unroll
  for (int t2 = 0; t2 < DTM; ++t2) o[t2] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = ex.sink, l = qd == 0 && ex.sink > -INFINITY ? 1.f : 0.f;
  const int p_min = ctx0 + r0, p_max = ctx0 + r0 + rows - 1;
  const int lo_min = first_visible(p_min, window, ex.chunked);
  const int row_lo = first_visible(qpos, window, ex.chunked);
  int ns = window > 0 ? min(keep_first, lo_min) : 0;
  const bool pooled = EXT && ex.pool > 0;
  if (pooled) ns = pooled_count(p_max, window, ex.pool);     // what the last row sees
  const bool halves = EXT && ex.vtab != nullptr && !ex.vinter;
  const int nsink = (ns + PFW_BN - 1) / PFW_BN;
  const int nmain = (p_max - lo_min + PFW_BN) / PFW_BN;
  // the wave's own span of visible keys (tiles outside it are staged but not computed)
  const int wp_lo = ctx0 + r0 + 16 * wave, wp_hi = min(wp_lo + 15, p_max);
  const int w_lo = first_visible(wp_lo, window, ex.chunked);
  const int w_lo_hi = first_visible(wp_hi, window, ex.chunked);
  const int keyA = 8 * (r16 >> 2) + (r16 & 3);
  const int kchunks = kp >> 3, vchunks = dv >> 3;
  const int bs_shift = (bs & (bs - 1)) == 0 ? __builtin_ctz(bs) : -1;
  auto page_row = [&](int key) -> int64_t {
    const int pg = bs_shift >= 0 ? key >> bs_shift : key / bs;
    const int in = bs_shift >= 0 ? key & (bs - 1) : key - pg * bs;
    int bl = bt[pg];
    if (bl < 0 || bl >= num_blocks) bl = 0;
    return (int64_t)(bl * G + g) * (EXT ? ex.prow : bs) + in;
  };
  auto block_row = [&](int b) -> int64_t {
    int pg, pr;
    pooled_place(b, ex.pool, bs, pg, pr);
    int bl = bt[pg];
    if (bl < 0 || bl >= num_blocks) bl = 0;
    return (int64_t)(bl * G + g) * ex.prow + pr;
  };
  const int sr = threadIdx.x >> 4, sc = threadIdx.x & 15;     // K staging: 16 lanes per key row
  for (int tile = 0; tile < nsink + nmain; ++tile) {
    const bool sink = tile < nsink, ptile = pooled && sink;
    const int kb = sink ? tile * PFW_BN : lo_min + (tile - nsink) * PFW_BN;
    const int hi = sink ? min(ns, kb + PFW_BN) : min(p_max + 1, kb + PFW_BN);
    __syncthreads();                         // the previous tile's fragments were read
#pragma unroll
    for (int kq = 0; kq < 4; ++kq) {
      const int ks = sr + 16 * kq, key = kb + ks;
      const T* src = key < hi ? k_cache + (ptile ? block_row(key) : page_row(key)) * krs : nullptr;
      for (int c = sc; c < kchunks; c += 16) {
        u32x4 val = u32x4{0u, 0u, 0u, 0u};
        if (src != nullptr && 8 * c < dk) val = *reinterpret_cast<const u32x4*>(src + 8 * c);
        *reinterpret_cast<u32x4*>(Ks + ks * kst + 8 * c) = val;
      }
    }
    {
      const int ks = threadIdx.x & (PFW_BN - 1), key = kb + ks;   // a wave's lanes: consecutive keys
      const T* src = key < hi ? v_cache + (ptile ? block_row(key) : page_row(key)) * vrs : nullptr;
      for (int c = threadIdx.x >> 6; c < vchunks; c += 4) {
        Pack8<T> val;
        val.u = u32x4{0u, 0u, 0u, 0u};
        if (src != nullptr) val.u = *reinterpret_cast<const u32x4*>(src + 8 * c);
        int r = 8 * c;
        if constexpr (EXT) {
          if (halves) {
            const int hf = r >= (dv >> 1), cc = hf ? r - (dv >> 1) : r;
            r = (cc >> 4) * 32 + 16 * hf + (cc & 15);
          }
        }
#pragma unroll
        for (int e2 = 0; e2 < 8; ++e2) Vt[(r + e2) * vst + ks] = val.h[e2];
      }
    }
    __syncthreads();
    if (16 * wave >= rows) continue;                       // no rows in this wave
    // nothing of this tile is visible to the wave's rows (kept first tokens can sit in a
    // main tile when the earliest window starts before them)
    if (ptile ? kb >= pooled_count(wp_hi, window, ex.pool)
              : kb > wp_hi || (!sink && hi <= w_lo && kb >= keep_first))
      continue;
    // ---- S^T tiles j = 0..3: keys 32 (j >> 1) + keyA + 4 (j & 1)
    f32x4 s[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const T* krow = Ks + ((j >> 1) * 32 + keyA + 4 * (j & 1)) * kst + 8 * qd;
      f32x4 a = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s2 = 0; s2 < KSM; ++s2) {
        if (s2 < nks) {
          Pack8<T> fr;
          fr.u = *reinterpret_cast<const u32x4*>(krow + 32 * s2);
          a = mfma16x16x32(fr.v, qf[s2], a);
        }
      }
      s[j] = a;
    }
    // ---- visibility and online softmax (query = lane & 15).  A tile whose 64 keys are
    // all valid, not after the wave's first row and inside the window of its last row is
    // seen in full by every row of the wave: no per-element test.
    const int nblk = ptile ? pooled_count(qpos, window, ex.pool) : 0;
    const bool full = ptile ? kb + PFW_BN <= pooled_count(wp_lo, window, ex.pool) && wp_lo + 15 == wp_hi
                            : hi == kb + PFW_BN && kb + PFW_BN - 1 <= wp_lo &&
                                  kb >= w_lo_hi && wp_lo + 15 == wp_hi;
    float tmax = -INFINITY;
    if (full) {
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          s[j][i] = cap_score(s[j][i] * scale, ex.softcap);
          tmax = fmaxf(tmax, s[j][i]);
        }
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int key = kb + (j >> 1) * 32 + 8 * qd + 4 * (j & 1) + i;
          const bool vis = ptile ? rowok && key < nblk
                                 : rowok && key < hi && key <= qpos &&
                                       (key >= row_lo || key < keep_first);
          s[j][i] = vis ? cap_score(s[j][i] * scale, ex.softcap) : -INFINITY;
          tmax = fmaxf(tmax, s[j][i]);
        }
    }
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
    const float mn = fmaxf(m, tmax);
    const float alpha = m == -INFINITY ? 0.f : __expf(m - mn);
    m = mn;
    l *= alpha;
    V8 phi[2], plo[2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      Pack8<T> ph, pl;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float pa = s[2 * kk][i] == -INFINITY ? 0.f : __expf(s[2 * kk][i] - mn);
        const float pb2 = s[2 * kk + 1][i] == -INFINITY ? 0.f : __expf(s[2 * kk + 1][i] - mn);
        l += pa + pb2;
        ph.h[i] = from_f<T>(pa);
        ph.h[4 + i] = from_f<T>(pb2);
        pl.h[i] = from_f<T>(pa - to_f(ph.h[i]));
        pl.h[4 + i] = from_f<T>(pb2 - to_f(ph.h[4 + i]));
      }
      phi[kk] = ph.v;
      plo[kk] = pl.v;
    }
    // ---- O^T += V^T . P^T
#pragma unroll
    for (int t2 = 0; t2 < DTM; ++t2) {
      if (t2 < ndt) {
        f32x4 acc = o[t2] * alpha;
        const T* vrow = Vt + (16 * t2 + r16) * vst + 8 * qd;
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
          Pack8<T> fr;
          fr.u = *reinterpret_cast<const u32x4*>(vrow + 32 * kk);
          acc = mfma16x16x32(fr.v, phi[kk], acc);
          acc = mfma16x16x32(fr.v, plo[kk], acc);
        }
        o[t2] = acc;
      }
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (rowok) {
    const float gt = (gate != nullptr ? gate[(int64_t)(q0 + myrow) * H + h] : 1.f) * ex.out_scale;
    const float inv = l > 0.f ? gt / l : 0.f;
    T* orow = out + (int64_t)(q0 + myrow) * ex.ors + h * dv;
    if constexpr (EXT) {
      if (ex.vtab != nullptr) {
        const float* cs = rot_row(ex, qpos, dv);
        const int half = dv >> 1;
        if (halves) {
#pragma unroll
          for (int t2 = 0; t2 < DTM; t2 += 2) {
            if (t2 < ndt) {
              const int m0 = 8 * t2 + 4 * qd;              // 16 (t2 / 2) + 4 qd
#pragma unroll
              for (int i = 0; i < 4; ++i) {
                const float a = o[t2][i], b = o[t2 + 1][i], c = cs[m0 + i], sn = cs[half + m0 + i];
                o[t2][i] = a * c + b * sn;
                o[t2 + 1][i] = b * c - a * sn;
              }
            }
          }
        } else {
#pragma unroll
          for (int t2 = 0; t2 < DTM; ++t2) {
            if (t2 < ndt) {
              const int m0 = 8 * t2 + 2 * qd;
#pragma unroll
              for (int i = 0; i < 4; i += 2) {
                const float a = o[t2][i], b = o[t2][i + 1];
                const float c = cs[m0 + (i >> 1)], sn = cs[half + m0 + (i >> 1)];
                o[t2][i] = a * c + b * sn;
                o[t2][i + 1] = b * c - a * sn;
              }
            }
          }
        }
      }
    }
#pragma unroll
    for (int t2 = 0; t2 < DTM; ++t2) {
      if (t2 < ndt) {
        const int c0 = halves ? (t2 & 1) * (dv >> 1) + 16 * (t2 >> 1) + 4 * qd : 16 * t2 + 4 * qd;
        Pack4<T> w4;
#pragma unroll
        for (int i = 0; i < 4; ++i)
          w4.h[i] = from_f<T>(o[t2][i] * inv * elem_gate<T>(ex, q0 + myrow, h * dv + c0 + i));
        *reinterpret_cast<u32x2*>(orow + c0) = w4.u;
      }
    }
  }
}

// VEC consecutive elements as fp32 / from fp32 (VEC 8: 16-byte accesses of 16-bit types)
template <typename T, int VEC>
__device__ __forceinline__ void load_vec(const T* p, float (&v)[VEC]) {
  if constexpr (VEC == 8) load8(p, v);
  else v[0] = to_f(p[0]);
}
template <typename T, int VEC>
__device__ __forceinline__ void store_vec(T* p, const float (&v)[VEC]) {
  if constexpr (VEC == 1) {
    p[0] = from_f<T>(v[0]);
  } else if constexpr (std::is_same_v<T, float>) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
  } else {
    Pack8<T> t;
#pragma unroll
    for (int e = 0; e < 8; ++e) t.h[e] = from_f<T>(v[e]);
    *reinterpret_cast<u32x4*>(p) = t.u;
  }
}

// norm_kv_store for head sizes that are multiples of 8 (<= 512) and 16-byte rows: 2^lsh lanes take
// one head vector, 8 adjacent elements each, and sum over themselves.
template <typename TI, typename T>
__global__ __launch_bounds__(256) void norm_kv_store_vec_kernel(
    const TI* __restrict__ qkv, int64_t qs, const int64_t* __restrict__ positions,
    T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache,
    const int64_t* __restrict__ slots, int H, int G, int dk, int dv, int bs, int num_blocks,
    float eps, bool qk_unit, bool v_unit, float coef, int every, const float* __restrict__ qw,
    const float* __restrict__ kw, int lsh) {
  const int64_t t = blockIdx.x;
  const TI* row = qkv + t * qs;
  int64_t pos = positions[t];
  if (pos < 0) pos = 0;
  const float temp = coef != 0.f ? 1.f + coef * logf((float)((pos + 1) / every) + 1.f) : 1.f;
  const int64_t slot = slots[t];
  const bool store = slot >= 0 && slot < (int64_t)num_blocks * bs;
  const int64_t blk = store ? slot / bs : 0, off = store ? slot % bs : 0;
  const int c = (threadIdx.x & ((1 << lsh) - 1)) * 8;
  const int nv = store ? H + 2 * G : H;
  for (int hv = threadIdx.x >> lsh; hv < nv; hv += 256 >> lsh) {
    const bool isq = hv < H, isk = !isq && hv < H + G;
    const int n = hv < H + G ? dk : dv;
    const TI* src = row + (hv < H + G ? hv * dk : (H + G) * dk + (hv - H - G) * dv);
    float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (c < n) load8(src + c, v);
    float f = isq ? temp : 1.f;
    if (isq || isk ? qk_unit : v_unit) {
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
      for (int o = 1; o < (1 << lsh); o <<= 1) ss += __shfl_xor(ss, o, 64);
      f /= sqrtf(ss / (float)n + eps);
    }
    if (c < n) {
      const float* w = isq ? qw : isk ? kw : nullptr;
      float wv[8];
      if (w != nullptr) {
        load8(w + c, wv);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] *= wv[e];
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] *= f;
      T* dst = isq ? q_out + (t * H + hv) * dk
                   : isk ? k_cache + ((blk * G + (hv - H)) * bs + off) * dk
                         : v_cache + ((blk * G + (hv - H - G)) * bs + off) * dv;
      store_vec<T, 8>(dst + c, v);
    }
  }
}

// One workgroup per token.  qkv row = q [H dk] (| k [G dk] | v [G dv] when a cache is given):
// the whole q row and the whole k row over their root mean squares times a weight per column,
// rotation of q and k on the first `rot` dims (table: cos | sin) and of v on all dv (vtab);
// q -> q_out [T, H, dk], k and v -> the cache row of the token's slot.  The row sits in LDS as
// fp32 between the sums and the outputs (STAGED), or is read again.  VEC 8: a thread makes 8 adjacent outputs (head sizes,
// rotated parts and strides are multiples that keep them in one head and one half).
template <typename T, int VEC, bool STAGED>
__global__ __launch_bounds__(256) void qk_norm_store_kernel(
    T* __restrict__ q_out, const T* __restrict__ qkv, int64_t qs, const int64_t* __restrict__ positions,
    const float* __restrict__ qw, const float* __restrict__ kw, const float* __restrict__ table,
    int rot, int trows, const float* __restrict__ vtab, int vrows, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const int64_t* __restrict__ slots, int H, int G, int dk, int dv,
    int bs, int prow, int num_blocks, float eps, bool inter) {
  extern __shared__ float lds[];
  __shared__ float scratch[4];
  const int64_t t = blockIdx.x;
  const T* row = qkv + t * qs;
  const int nq = H * dk, nk = k_cache != nullptr ? G * dk : 0, nv = k_cache != nullptr ? G * dv : 0;
  const int64_t slot = slots[t];
  const bool store = nk > 0 && slot >= 0 && slot < (int64_t)num_blocks * bs;
  const int n = nq + (store ? nk + nv : 0);
  float sq = 0.f, sk = 0.f;
  for (int e = threadIdx.x * VEC; e < n; e += 256 * VEC) {
    float v[VEC];
    load_vec<T, VEC>(row + e, v);
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      if constexpr (STAGED) lds[e + i] = v[i];
      ss += v[i] * v[i];
    }
    if (e < nq) sq += ss;
    else if (e < nq + nk) sk += ss;
  }
  sq = block_sum<256>(sq, scratch);
  if (store) sk = block_sum<256>(sk, scratch);
  const float rq = 1.f / sqrtf(sq / (float)nq + eps);
  const float rk = store ? 1.f / sqrtf(sk / (float)nk + eps) : 0.f;
  int64_t pos = positions[t];
  if (pos < 0) pos = 0;
  const float* cs = table != nullptr ? table + (pos < trows ? pos : trows - 1) * rot : nullptr;
  const float* vcs = vtab != nullptr ? vtab + (pos < vrows ? pos : vrows - 1) * dv : nullptr;
  const int64_t blk = store ? slot / bs : 0, off = store ? slot % bs : 0;
  for (int e = threadIdx.x * VEC; e < n; e += 256 * VEC) {
    const bool isv = e >= nq + nk, isq = e < nq;
    const int e0 = isq ? e : isv ? e - nq - nk : e - nq, hs = isv ? dv : dk;
    const int head = e0 / hs, i0 = e0 - head * hs;
    const float f = isq ? rq : isv ? 1.f : rk;
    const float* w = isq ? qw : kw;
    const float* rc = isv ? vcs : cs;
    const int rd = rc == nullptr ? 0 : isv ? dv : rot, half = rd >> 1;
    const int b0 = e - i0;                             // the head's first element
    auto val = [&](int i) {
      float x;
      if constexpr (STAGED) x = lds[b0 + i];
      else x = to_f(row[b0 + i]);
      return x * (isv ? 1.f : f * w[e0 - i0 + i]);
    };
    float v[VEC];
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      const int i = i0 + k;
      v[k] = val(i);
      if (i < rd) {
        const int p = inter ? i >> 1 : (i < half ? i : i - half);
        const bool first = inter ? !(i & 1) : i < half;
        const float o = val(inter ? i ^ 1 : (first ? i + half : i - half));
        const float c = rc[p], sn = rc[half + p];
        v[k] = first ? v[k] * c - o * sn : v[k] * c + o * sn;
      }
    }
    T* dst = isq ? q_out + t * nq + e
                 : isv ? v_cache + ((blk * G + head) * prow + off) * dv + i0
                       : k_cache + ((blk * G + head) * prow + off) * dk + i0;
    store_vec<T, VEC>(dst, v);
  }
}

// The same for head sizes, rotated parts and alignments that are multiples of 16 elements and
// pairs in halves: a thread owns NU units of two 8-element pieces that rotate into each other
// (or two adjacent pieces past the rotated part) and keeps them in registers between the sums
// and the outputs.
template <typename T, int NU>
__global__ __launch_bounds__(256) void qk_norm_store_pairs_kernel(
    T* __restrict__ q_out, const T* __restrict__ qkv, int64_t qs, const int64_t* __restrict__ positions,
    const float* __restrict__ qw, const float* __restrict__ kw, const float* __restrict__ table,
    int rot, int trows, const float* __restrict__ vtab, int vrows, T* __restrict__ k_cache,
    T* __restrict__ v_cache, const int64_t* __restrict__ slots, int H, int G, int dk, int dv,
    int bs, int prow, int num_blocks, float eps) {
  __shared__ float scratch[2][4];
  const int64_t t = blockIdx.x;
  const T* row = qkv + t * qs;
  const int64_t slot = slots[t];
  const bool store = k_cache != nullptr && slot >= 0 && slot < (int64_t)num_blocks * bs;
  const int uk = dk >> 4, uv = dv >> 4;                // units per head
  const int nq = H * uk, nk = store ? G * uk : 0, nv = store ? G * uv : 0;
  int64_t pos = positions[t];
  if (pos < 0) pos = 0;
  const float* cs = table != nullptr ? table + (pos < trows ? pos : trows - 1) * rot : nullptr;
  const float* vcs = vtab != nullptr ? vtab + (pos < vrows ? pos : vrows - 1) * dv : nullptr;
  float a[NU][8], b[NU][8], sq = 0.f, sk = 0.f;
  int hd[NU], oa[NU], ob[NU], ri[NU];                  // head, piece offsets in it, pair index or -1
#pragma unroll
  for (int n = 0; n < NU; ++n) {
    const int u = threadIdx.x + 256 * n;
    hd[n] = -1;
    if (u < nq + nk + nv) {
      const bool isv = u >= nq + nk, isq = u < nq;
      const int per = isv ? uv : uk, u0 = isq ? u : isv ? u - nq - nk : u - nq;
      const int h = u0 / per, i = u0 - h * per, rd = isv ? (vcs ? dv : 0) : (cs ? rot : 0);
      hd[n] = h;
      ri[n] = i < (rd >> 4) ? 8 * i : -1;
      oa[n] = ri[n] >= 0 ? 8 * i : 16 * i;
      ob[n] = ri[n] >= 0 ? (rd >> 1) + 8 * i : 16 * i + 8;
      const T* src = row + (isq ? h * dk : isv ? (H + G) * dk + h * dv : (H + h) * dk);
      load8(src + oa[n], a[n]);
      load8(src + ob[n], b[n]);
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) ss += a[n][e] * a[n][e] + b[n][e] * b[n][e];
      if (isq) sq += ss;
      else if (!isv) sk += ss;
    }
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
  const float rq = 1.f / sqrtf(sq / (float)(H * dk) + eps);
  const float rk = store ? 1.f / sqrtf(sk / (float)(G * dk) + eps) : 0.f;
  const int64_t blk = store ? slot / bs : 0, off = store ? slot % bs : 0;
#pragma unroll
  for (int n = 0; n < NU; ++n) {
    if (hd[n] < 0) continue;
    const int u = threadIdx.x + 256 * n, h = hd[n];
    const bool isv = u >= nq + nk, isq = u < nq;
    if (!isv) {
      const float* w = (isq ? qw : kw) + h * dk;
      const float f = isq ? rq : rk;
      float wa[8], wb[8];
      load8(w + oa[n], wa);
      load8(w + ob[n], wb);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        a[n][e] *= f * wa[e];
        b[n][e] *= f * wb[e];
      }
    }
    if (ri[n] >= 0) {
      const float* rc = isv ? vcs : cs;
      float c[8], sn[8];
      load8(rc + ri[n], c);
      load8(rc + ((isv ? dv : rot) >> 1) + ri[n], sn);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float x = a[n][e], y = b[n][e];
        a[n][e] = x * c[e] - y * sn[e];
        b[n][e] = y * c[e] + x * sn[e];
      }
    }
    T* dst = isq ? q_out + (t * H + h) * dk
                 : isv ? v_cache + ((blk * G + h) * prow + off) * dv
                       : k_cache + ((blk * G + h) * prow + off) * dk;
    store_vec<T, 8>(dst + oa[n], a[n]);
    store_vec<T, 8>(dst + ob[n], b[n]);
  }
}

// Blocks of `pool` tokens completed by prefill chunks: one workgroup per (work item of blk_rows
// chunk rows, kv head); a thread takes VEC adjacent columns of one block's key or value row.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void pool_chunks_kernel(
    T* k_cache, T* v_cache, const int64_t* __restrict__ slots, const int* __restrict__ qsl,
    const int* __restrict__ seq_lens, const int* __restrict__ pbt, int bt_stride,
    const int* __restrict__ work_seq, const int* __restrict__ work_blk, int blk_rows, int G, int dk,
    int dv, int krs, int vrs, int bs, int prow, int num_blocks, int pool) {
  const int seq = work_seq[blockIdx.x], g = blockIdx.y;
  const int q0 = qsl[seq], qlen = qsl[seq + 1] - q0, ctx0 = seq_lens[seq] - qlen;
  const int r0 = work_blk[blockIdx.x] * blk_rows;
  if (r0 >= qlen || ctx0 < 0) return;
  const int p0 = ctx0 + r0, p1 = ctx0 + min(qlen, r0 + blk_rows);     // positions [p0, p1)
  if (p1 > bt_stride * bs) return;
  const int* bt = pbt + (int64_t)seq * bt_stride;
  const int b0 = p0 / pool, nblk = p1 / pool - b0;                     // blocks ending in there
  const int kc = dk / VEC, nc = kc + dv / VEC;
  const float inv = 1.f / (float)pool;
  for (int it = threadIdx.x; it < nblk * nc; it += 256) {
    const int bl = it / nc, c = it - bl * nc, b = b0 + bl, last = b * pool + pool - 1;
    if (slots[q0 + last - ctx0] < 0) continue;
    T* base = c < kc ? k_cache + c * VEC : v_cache + (c - kc) * VEC;
    const int rs = c < kc ? krs : vrs;
    float acc[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] = 0.f;
    int pg = (last + 1 - pool) / bs, in = last + 1 - pool - pg * bs;
#pragma unroll 4
    for (int j = 0; j < pool; ++j) {
      int pb = bt[pg];
      if (pb < 0 || pb >= num_blocks) pb = 0;
      float v[VEC];
      load_vec<T, VEC>(base + ((int64_t)(pb * G + g) * prow + in) * rs, v);
#pragma unroll
      for (int e = 0; e < VEC; ++e) acc[e] += v[e];
      if (++in == bs) {
        in = 0;
        ++pg;
      }
    }
#pragma unroll
    for (int e = 0; e < VEC; ++e) acc[e] *= inv;
    int dp, dr;
    pooled_place(b, pool, bs, dp, dr);
    int db = bt[dp];
    if (db < 0 || db >= num_blocks) db = 0;
    store_vec<T, VEC>(base + ((int64_t)(db * G + g) * prow + dr) * rs, acc);
  }
}

// Rows t0 .. of a step that complete a block of `pool` tokens (and are stored) write the
// block's mean rows; grid (rows, G).
template <typename T>
__global__ __launch_bounds__(256) void pool_kv_kernel(
    T* k_cache, T* v_cache, const int64_t* __restrict__ slots, const int* __restrict__ qsl,
    const int* __restrict__ seq_lens, const int* __restrict__ pbt, const int* __restrict__ ctx_lens,
    const int* __restrict__ dbt, int bt_stride, int P, int Tp, int t0, int G, int dk, int dv,
    int krs, int vrs, int bs, int prow, int num_blocks, int pool) {
  const int t = t0 + blockIdx.x;
  if (slots[t] < 0) return;
  int pos;
  const int* bt;
  if (t < Tp) {
    int lo = 0, hi = P - 1;
    while (lo < hi) {
      const int mid = (lo + hi + 1) >> 1;
      if (qsl[mid] <= t) lo = mid; else hi = mid - 1;
    }
    pos = seq_lens[lo] - (qsl[lo + 1] - qsl[lo]) + (t - qsl[lo]);
    bt = pbt + (int64_t)lo * bt_stride;
  } else {
    pos = ctx_lens[t - Tp] - 1;
    bt = dbt + (int64_t)(t - Tp) * bt_stride;
  }
  if (pos < 0 || pos >= bt_stride * bs || (pos + 1) % pool != 0) return;
  pool_block<T>(k_cache, v_cache, bt, pos, pool, blockIdx.y, G, dk, dv, krs, vrs, bs, prow,
                num_blocks, threadIdx.x, 256);
}

}  // namespace

#define KGC_DISPATCH_T(dtype, ...)                          \
  do {                                                      \
    if ((dtype) == DT_BF16) { typedef bf16 T; __VA_ARGS__; } \
    else if ((dtype) == DT_F16) { typedef f16 T; __VA_ARGS__; } \
    else { typedef float T; __VA_ARGS__; }                  \
  } while (0)

void launch_rope_kv_store(int dtype, const void* qkv, int64_t qkv_stride,
                          const int64_t* positions, const float* table, int rot, int table_rows,
                          void* q_out, void* k_cache, void* v_cache, const int64_t* slots, int T_,
                          int H, int G, int dk, int dv, int bs, int num_blocks, bool interleaved,
                          hipStream_t s) {
  if (T_ <= 0) return;
  KGC_DISPATCH_T(dtype, rope_kv_store_kernel<T><<<T_, 256, 0, s>>>(
      (const T*)qkv, qkv_stride, positions, table, rot, table_rows, (T*)q_out, (T*)k_cache,
      (T*)v_cache, slots, H, G, dk, dv, bs, num_blocks, interleaved));
}

void launch_norm_kv_store(int dtype, int out_dtype, const void* qkv, int64_t qs,
                          const int64_t* positions, void* q_out, void* k_cache, void* v_cache,
                          const int64_t* slots, int T_, int H, int G, int dk, int dv, int bs,
                          int num_blocks, float eps, bool qk_unit, bool v_unit, float coef,
                          int every, const float* qw, const float* kw, hipStream_t s) {
  if (T_ <= 0) return;
  auto al = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  const bool vec = dk % 8 == 0 && dv % 8 == 0 && dk <= 512 && dv <= 512 &&
                   qs % (dtype == DT_F32 ? 4 : 8) == 0 && al(qkv) && al(q_out) && al(k_cache) &&
                   al(v_cache) && al(qw) && al(kw);
  int lsh = 0;
  while ((8 << lsh) < std::max(dk, dv)) ++lsh;
#define KGC_NKV(TI)                                                                             \
  do {                                                                                          \
    if (vec)                                                                                    \
      norm_kv_store_vec_kernel<TI, T><<<T_, 256, 0, s>>>(                                       \
          (const TI*)qkv, qs, positions, (T*)q_out, (T*)k_cache, (T*)v_cache, slots, H, G, dk, dv, \
          bs, num_blocks, eps, qk_unit, v_unit, coef, every, qw, kw, lsh);                      \
    else                                                                                        \
      norm_kv_store_kernel<TI, T><<<T_, 256, 0, s>>>(                                           \
          (const TI*)qkv, qs, positions, (T*)q_out, (T*)k_cache, (T*)v_cache, slots, H, G, dk, dv, \
          bs, num_blocks, eps, qk_unit, v_unit, coef, every, qw, kw);                           \
  } while (0)
  if (dtype == DT_F32) KGC_DISPATCH_T(out_dtype, KGC_NKV(float));
  else KGC_DISPATCH_T(out_dtype, KGC_NKV(T));
#undef KGC_NKV
}

void launch_qk_norm_store(int dtype, void* q_out, const void* qkv, int64_t qs,
                          const int64_t* positions, const float* qw, const float* kw,
                          const float* table, int rot, int trows, const float* vtab, int vrows,
                          void* k_cache, void* v_cache, const int64_t* slots, int T_, int H, int G,
                          int dk, int dv, int bs, int prow, int num_blocks, float eps, bool inter,
                          hipStream_t s) {
  if (T_ <= 0) return;
  const bool kv = k_cache != nullptr;
  const size_t row_lds = sizeof(float) * (size_t)(H * dk + (kv ? G * (dk + dv) : 0));
  const bool staged = row_lds <= 64 * 1024;
  const size_t lds = staged ? row_lds : 0;
  // eight adjacent elements of one head and one half of the rotated part, 16-byte aligned
  const bool vec = dk % 8 == 0 && (!kv || dv % 8 == 0) && qs % 8 == 0 &&
                   reinterpret_cast<uintptr_t>(qkv) % 16 == 0;
  const int units = (H * dk + (kv ? G * (dk + dv) : 0)) / 16;
  if (vec && !inter && dk % 16 == 0 && (!kv || dv % 16 == 0) && rot % 16 == 0 && units <= 1024 &&
      reinterpret_cast<uintptr_t>(qw) % 16 == 0 && reinterpret_cast<uintptr_t>(kw) % 16 == 0) {
#define KGC_QKP(N)                                                                           \
  KGC_DISPATCH_T(dtype, qk_norm_store_pairs_kernel<T, N><<<T_, 256, 0, s>>>(                 \
      (T*)q_out, (const T*)qkv, qs, positions, qw, kw, table, rot, trows, vtab, vrows,       \
      (T*)k_cache, (T*)v_cache, slots, H, G, dk, dv, bs, prow, num_blocks, eps))
    if (units <= 256) KGC_QKP(1);
    else if (units <= 512) KGC_QKP(2);
    else KGC_QKP(4);
#undef KGC_QKP
    return;
  }
#define KGC_QKN(V, ST)                                                                       \
  KGC_DISPATCH_T(dtype, qk_norm_store_kernel<T, V, ST><<<T_, 256, lds, s>>>(                 \
      (T*)q_out, (const T*)qkv, qs, positions, qw, kw, table, rot, trows, vtab, vrows,       \
      (T*)k_cache, (T*)v_cache, slots, H, G, dk, dv, bs, prow, num_blocks, eps, inter))
  if (!staged) KGC_QKN(1, false);
  else if (vec) KGC_QKN(8, true);
  else KGC_QKN(1, true);
#undef KGC_QKN
}

void launch_pool_kv(int dtype, void* k_cache, void* v_cache, const int64_t* slots, const int* qsl,
                    const int* seq_lens, const int* pbt, const int* ctx_lens, const int* dbt,
                    int bt_stride, int P, int Tp, int t0, int rows, int G, int dk, int dv, int krs,
                    int vrs, int bs, int prow, int num_blocks, int pool, hipStream_t s) {
  if (rows <= 0) return;
  KGC_DISPATCH_T(dtype, pool_kv_kernel<T><<<dim3(rows, G), 256, 0, s>>>(
      (T*)k_cache, (T*)v_cache, slots, qsl, seq_lens, pbt, ctx_lens, dbt, bt_stride, P, Tp, t0, G,
      dk, dv, krs, vrs, bs, prow, num_blocks, pool));
}

void launch_pool_chunks(int dtype, void* k_cache, void* v_cache, const int64_t* slots,
                        const int* qsl, const int* seq_lens, const int* pbt, int bt_stride,
                        const int* work_seq, const int* work_blk, int n_work, int blk_rows, int G,
                        int dk, int dv, int krs, int vrs, int bs, int prow, int num_blocks,
                        int pool, hipStream_t s) {
  if (n_work <= 0) return;
#define KGC_PC(V)                                                                            \
  KGC_DISPATCH_T(dtype, pool_chunks_kernel<T, V><<<dim3(n_work, G), 256, 0, s>>>(            \
      (T*)k_cache, (T*)v_cache, slots, qsl, seq_lens, pbt, bt_stride, work_seq, work_blk,    \
      blk_rows, G, dk, dv, krs, vrs, bs, prow, num_blocks, pool))
  if (dk % 8 == 0 && dv % 8 == 0 && krs % 8 == 0 && vrs % 8 == 0) KGC_PC(8); else KGC_PC(1);
#undef KGC_PC
}

int window_attention_max_dv() { return 64 * MAX_DV_PER_LANE; }

void launch_window_attention(int dtype, void* out, const void* q, const void* k_cache,
                             const void* v_cache, const int* qsl, const int* seq_lens,
                             const int* pbt, const int* ctx_lens, const int* dbt, int bt_stride,
                             int P, int Tp, int T_, int H, int G, int dk, int dv, int krs, int vrs,
                             int bs, int num_blocks, float scale, int window, int keep_first,
                             const float* gate, int kinds, WindowExtra ex, hipStream_t s) {
  if (T_ <= 0 || !kinds) return;
  const size_t lds = (size_t)(dk + 128 + (ex.vtab != nullptr ? dv : 0)) * sizeof(float);
  KGC_DISPATCH_T(dtype, window_attention_kernel<T><<<dim3(T_, H), 64, lds, s>>>(
      (T*)out, (const T*)q, (const T*)k_cache, (const T*)v_cache, qsl, seq_lens, pbt, ctx_lens,
      dbt, bt_stride, P, Tp, H, G, dk, dv, krs, vrs, bs, num_blocks, scale, window, keep_first,
      gate, kinds, ex));
}

// decode rows on the 8-wave kernel: needs 16-byte key rows (dk % 8 == 0), even dv <= 512
bool window_decode_ok(int dk, int dv, int qpg) {
  (void)qpg;
  return dk % 8 == 0 && dv % 2 == 0 && dv <= 128 * DEC_UMAX;
}

static size_t decode_lds(int QH, int nwv, int dk, int dv) {
  return sizeof(float) * ((size_t)QH * dk + (size_t)nwv * QH * 64 + nwv * 64 + 2 * nwv * QH +
                          (size_t)QH * dv);
}

template <typename T>
static void decode_dispatch(T* out, const T* q, const T* kc, const T* vc, const int* ctx_lens,
                            const int* dbt, int bt_stride, int Tp, int D, int H, int G, int dk,
                            int dv, int krs, int vrs, int bs, int num_blocks, float scale, int window,
                            int keep_first, const float* gate, WindowExtra ex, hipStream_t s) {
  const int qpg = H / G;
  int QH = qpg >= 8 ? 8 : qpg >= 3 ? 4 : qpg;            // heads per workgroup: 1, 2, 4, 8
  // many heads on one key/value group and few rows: smaller head groups, so that the grid
  // still covers the CUs (the groups re-read the rows from L2)
  while (QH > 2 && (int64_t)D * G * ((qpg + QH - 1) / QH) < 256) QH >>= 1;
  const dim3 grid(D, G, (qpg + QH - 1) / QH);
  // 8 waves split a row's keys finest (shortest chain per workgroup); once the grid holds
  // two workgroups per CU, 4-wave workgroups let two of them overlap on a CU instead
  const bool small = (int64_t)grid.x * grid.y * grid.z >= 512;
  const bool ext = ex.pool > 0 || ex.vtab != nullptr;
#define KGC_DEC_E(N, W, E)                                                                   \
  window_decode_kernel<T, N, W, E><<<grid, 64 * W, decode_lds(N, W, dk, dv), s>>>(           \
      out, q, kc, vc, ctx_lens, dbt, bt_stride, Tp, H, G, dk, dv, krs, vrs, bs, num_blocks,     \
      scale, window, keep_first, gate, ex)
#define KGC_DEC(N, W)                                         \
  do {                                                        \
    if (ext) KGC_DEC_E(N, W, true); else KGC_DEC_E(N, W, false); \
  } while (0)
#define KGC_DEC2(N) \
  do {              \
    if (small) KGC_DEC(N, 4); else KGC_DEC(N, 8); \
  } while (0)
  if (QH == 8) KGC_DEC2(8);
  else if (QH == 4) KGC_DEC2(4);
  else if (QH == 2) KGC_DEC2(2);
  else KGC_DEC2(1);
#undef KGC_DEC2
#undef KGC_DEC
#undef KGC_DEC_E
}

size_t window_decode_lds(int dk, int dv, int qpg) {
  const int QH = qpg >= 8 ? 8 : qpg >= 3 ? 4 : qpg;
  return decode_lds(QH, DEC_WAVES, dk, dv);
}

void launch_window_decode(int dtype, void* out, const void* q, const void* k_cache,
                          const void* v_cache, const int* ctx_lens, const int* dbt,
                          int bt_stride, int Tp, int D, int H, int G, int dk, int dv, int krs,
                          int vrs, int bs, int num_blocks, float scale, int window, int keep_first,
                          const float* gate, WindowExtra ex, hipStream_t s) {
  if (D <= 0) return;
  KGC_DISPATCH_T(dtype, decode_dispatch<T>((T*)out, (const T*)q, (const T*)k_cache,
                                           (const T*)v_cache, ctx_lens, dbt, bt_stride, Tp, D, H,
                                           G, dk, dv, krs, vrs, bs, num_blocks, scale, window, keep_first,
                                           gate, ex, s));
}

// (with one or two query heads per key/value head the vector kernel is as fast)
bool window_decode_mfma_ok(int dtype, int dk, int dv, int qpg, const WindowExtra& ex) {
  return (dtype == DT_BF16 || dtype == DT_F16) && dk % 8 == 0 && dk <= 256 && dv % 8 == 0 &&
         dv <= 256 && qpg >= 3 && ex.pool == 0 && ex.vtab == nullptr;
}

template <typename T>
static void decode_mfma_dispatch(T* out, const T* q, const T* kc, const T* vc, const int* ctx_lens,
                                 const int* dbt, int bt_stride, int Tp, int D, int H, int G, int dk,
                                 int dv, int krs, int vrs, int bs, int num_blocks, float scale,
                                 int window, int keep_first, const float* gate, WindowExtra ex,
                                 hipStream_t s) {
  const dim3 grid(D, G, (H / G + 15) / 16);
  const bool shared = kc == vc && krs == vrs && dv <= dk;
  const bool small = (int64_t)grid.x * grid.y * grid.z >= 512;     // several workgroups per CU
#define KGC_DM(K, D_, W)                                                                       \
  window_decode_mfma_kernel<T, K, D_, W><<<grid, 64 * W, 0, s>>>(                              \
      out, q, kc, vc, ctx_lens, dbt, bt_stride, Tp, H, G, dk, dv, krs, vrs, bs, num_blocks, scale, \
      window, keep_first, gate, shared, ex)
#define KGC_DM2(K, D_)                              \
  do {                                              \
    if (small) KGC_DM(K, D_, 4); else KGC_DM(K, D_, 8); \
  } while (0)
  if (dk <= 128 && dv <= 128) KGC_DM2(4, 8);
  else if (dv <= 192) KGC_DM2(8, 12);
  else KGC_DM(8, 16, 4);
#undef KGC_DM2
#undef KGC_DM
}

void launch_window_decode_mfma(int dtype, void* out, const void* q, const void* k_cache,
                               const void* v_cache, const int* ctx_lens, const int* dbt,
                               int bt_stride, int Tp, int D, int H, int G, int dk, int dv, int krs,
                               int vrs, int bs, int num_blocks, float scale, int window,
                               int keep_first, const float* gate, WindowExtra ex, hipStream_t s) {
  if (D <= 0) return;
  if (dtype == DT_BF16)
    decode_mfma_dispatch<bf16>((bf16*)out, (const bf16*)q, (const bf16*)k_cache,
                               (const bf16*)v_cache, ctx_lens, dbt, bt_stride, Tp, D, H, G, dk, dv,
                               krs, vrs, bs, num_blocks, scale, window, keep_first, gate, ex, s);
  else
    decode_mfma_dispatch<f16>((f16*)out, (const f16*)q, (const f16*)k_cache, (const f16*)v_cache,
                              ctx_lens, dbt, bt_stride, Tp, D, H, G, dk, dv, krs, vrs, bs,
                              num_blocks, scale, window, keep_first, gate, ex, s);
}

size_t window_prefill_mfma_lds(int dk, int dv) {
  return 2 * ((size_t)PFW_BN * (((dk + 31) & ~31) + PFW_KPAD) + (size_t)dv * (PFW_BN + PFW_VPAD));
}

// the matrix-core prefill path: 16-bit activations, dk a multiple of 8 (<= 256), dv a
// multiple of 16 (<= 256), both tiles within 64 KB of LDS
bool window_prefill_mfma_ok(int dtype, int dk, int dv) {
  return (dtype == DT_BF16 || dtype == DT_F16) && dk % 8 == 0 && dk <= 256 && dv % 16 == 0 &&
         dv <= 256 && window_prefill_mfma_lds(dk, dv) <= 64 * 1024;
}

template <typename T>
static void prefill_dispatch(T* out, const T* q, const T* kc, const T* vc, const int* qsl,
                             const int* seq_lens, const int* pbt, int bt_stride,
                             const int* work_seq, const int* work_blk, int n_work, int blk_rows,
                             int H, int G, int dk, int dv, int krs, int vrs, int bs, int num_blocks,
                             float scale, int window, int keep_first, const float* gate,
                             WindowExtra ex, hipStream_t s) {
  const dim3 grid(H, n_work * (blk_rows / PFW_BM));
  const size_t lds = window_prefill_mfma_lds(dk, dv);
  const bool ext = ex.pool > 0 || ex.vtab != nullptr;
#define KGC_PF_E(K, D, E)                                                                     \
  window_prefill_mfma_kernel<T, K, D, E><<<grid, 256, lds, s>>>(                              \
      out, q, kc, vc, qsl, seq_lens, pbt, bt_stride, work_seq, work_blk, blk_rows, H, G, dk,  \
      dv, krs, vrs, bs, num_blocks, scale, window, keep_first, gate, ex)
#define KGC_PF(K, D)                                       \
  do {                                                     \
    if (ext) KGC_PF_E(K, D, true); else KGC_PF_E(K, D, false); \
  } while (0)
  if (dk <= 128 && dv <= 128) KGC_PF(4, 8);
  else KGC_PF(8, 16);
#undef KGC_PF
#undef KGC_PF_E
}

void launch_window_prefill_mfma(int dtype, void* out, const void* q, const void* k_cache,
                                const void* v_cache, const int* qsl, const int* seq_lens,
                                const int* pbt, int bt_stride, const int* work_seq,
                                const int* work_blk, int n_work, int blk_rows, int H, int G,
                                int dk, int dv, int krs, int vrs, int bs, int num_blocks, float scale, int window,
                                int keep_first, const float* gate, WindowExtra ex, hipStream_t s) {
  if (n_work <= 0) return;
  if (dtype == DT_BF16)
    prefill_dispatch<bf16>((bf16*)out, (const bf16*)q, (const bf16*)k_cache,
                           (const bf16*)v_cache, qsl, seq_lens, pbt, bt_stride, work_seq,
                           work_blk, n_work, blk_rows, H, G, dk, dv, krs, vrs, bs, num_blocks,
                           scale, window, keep_first, gate, ex, s);
  else
    prefill_dispatch<f16>((f16*)out, (const f16*)q, (const f16*)k_cache, (const f16*)v_cache,
                          qsl, seq_lens, pbt, bt_stride, work_seq, work_blk, n_work, blk_rows, H,
                          G, dk, dv, krs, vrs, bs, num_blocks, scale, window, keep_first, gate, ex, s);
}

// ---- latent attention: cache rows [normed latent | rotary key part] and query rows --------
namespace {

// One workgroup per token.  proj row: per head [d unrotated | r rotary] query columns, then
// the latent pre-activation (rank) and the shared rotary key part (r).  q_lat [H, T, rank]
// holds the unrotated query parts already multiplied into latent space.
//   q_out [T, H, rank + r] = [q_lat | rotated query part]
//   cache row (slot)       = [latent / rms(latent) * nw | rotated key part]
// Rotary pairs are (2i, 2i + 1); table row = cos[r/2] | sin[r/2], fp32.
template <typename T>
__global__ __launch_bounds__(256) void latent_rope_store_kernel(
    T* __restrict__ q_out, const T* __restrict__ proj, int64_t proj_stride,
    const T* __restrict__ q_lat, const int64_t* __restrict__ positions,
    const float* __restrict__ table, int table_rows, const float* __restrict__ nw, float eps,
    T* __restrict__ cache, const int64_t* __restrict__ slots, int64_t cache_rows, int T_, int H,
    int d, int r, int rank) {
  __shared__ float scratch[4];
  const int64_t t = blockIdx.x;
  const T* row = proj + t * proj_stride;
  int64_t pos = positions[t];
  if (pos < 0) pos = 0;
  if (pos >= table_rows) pos = table_rows - 1;        // host checks max_pos; never read past
  const float* cs = table != nullptr ? table + pos * r : nullptr;
  const int half = r >> 1, dq = d + r, dk = rank + r;
  for (int e = threadIdx.x; e < H * dk; e += 256) {
    const int head = e / dk, i = e - head * dk;
    float v;
    if (i < rank) {
      v = to_f(q_lat[((int64_t)head * T_ + t) * rank + i]);
    } else {
      const int j = i - rank, p = j >> 1;
      const T* qr = row + head * dq + d;
      float oa, ob;
      neox_rot(to_f(qr[2 * p]), to_f(qr[2 * p + 1]), cs[p], cs[half + p], oa, ob);
      v = (j & 1) ? ob : oa;
    }
    q_out[t * H * dk + e] = from_f<T>(v);
  }
  const int64_t slot = slots[t];
  const T* kv = row + (int64_t)H * dq;
  float ss = 0.f;
  for (int c = threadIdx.x; c < rank; c += 256) {
    const float v = to_f(kv[c]);
    ss += v * v;
  }
  ss = block_sum<256>(ss, scratch);
  if (slot < 0 || slot >= cache_rows) return;
  const float rn = 1.f / sqrtf(ss / (float)rank + eps);
  T* crow = cache + slot * dk;
  for (int c = threadIdx.x; c < dk; c += 256) {
    float v;
    if (c < rank) {
      v = to_f(kv[c]) * rn * nw[c];
    } else {
      const int j = c - rank, p = j >> 1;
      float oa, ob;
      neox_rot(to_f(kv[rank + 2 * p]), to_f(kv[rank + 2 * p + 1]), cs[p], cs[half + p], oa, ob);
      v = (j & 1) ? ob : oa;
    }
    crow[c] = from_f<T>(v);
  }
}

}  // namespace

void launch_latent_rope_store(int dtype, void* q_out, const void* proj, int64_t proj_stride,
                              const void* q_lat, const int64_t* positions, const float* table,
                              int table_rows, const float* nw, float eps, void* cache,
                              const int64_t* slots, int64_t cache_rows, int T_, int H, int d,
                              int r, int rank, hipStream_t s) {
  if (T_ <= 0) return;
  KGC_DISPATCH_T(dtype, latent_rope_store_kernel<T><<<T_, 256, 0, s>>>(
      (T*)q_out, (const T*)proj, proj_stride, (const T*)q_lat, positions, table, table_rows, nw,
      eps, (T*)cache, slots, cache_rows, T_, H, d, r, rank));
}

}  // namespace kgc
