// What the residual stream is still to get, and what the next part reads of it, in one pass over the rows:
//
//   s = x + sum over the plain terms of f y + sum over the normed terms of f (y / sqrt(mean(y^2) + eps)) w
//   (kept as `result` if asked for; also rounded to the activation type, for a product that reads the stream itself)
//   u = s, or with an average over the depth  u = c[0] first + sum_j c[1 + j] past[j] + c[last] s   (kept as `xout`)
//   h_k = (u / sqrt(mean(u^2) + eps_k)) w_k  for up to two norms of the same row
//
// A term y is rows in either precision or a stack of float32 partial sums, added in order.  Everything is float32 but
// the stores of `rounded` and h_k.  x null: zeros.  `rows`: only those rows are made (x, terms and past are read there).
// A normed term and a norm may each be made in groups: the row falls into that many equal parts, each divided by its own
// root mean square; the weight is as long as the row.
// Every operand is read before the row is written, and no output may be an input.
#include "common.h"

namespace xi {

constexpr int kJoinPlain = 3, kJoinNormed = 2, kJoinNorms = 2;
constexpr int kJoinGroups = 256;      // most groups of a norm

struct JoinTerm {
  const void* y = nullptr;
  size_t part_stride = 0;
  const float* w = nullptr;      // normed terms
  int parts = 1, dtype = kF32;
  float eps = 0.f, factor = 1.f;
  int groups = 1;                // normed terms
};

struct JoinArgs {
  const float* x;
  JoinTerm plain[kJoinPlain], normed[kJoinNormed];
  int n_plain, n_normed;
  float* result;
  void* rounded;
  const float* first;            // null: no average
  const float* past;
  size_t past_stride;
  int n_past;
  const float* coef;
  float* xout;
  const float* w[kJoinNorms];
  float eps[kJoinNorms];
  int groups[kJoinNorms];
  void* h[kJoinNorms];
  int n_norms;
  const int* rows;
  int H;
};

struct alignas(8) join_bf16x4 { bf16 v[4]; };
static __device__ __forceinline__ float4 join_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
static __device__ __forceinline__ float4 join_load4(const bf16* p) {
  const join_bf16x4 t = *reinterpret_cast<const join_bf16x4*>(p);
  return float4{to_float(t.v[0]), to_float(t.v[1]), to_float(t.v[2]), to_float(t.v[3])};
}
static __device__ __forceinline__ void join_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
static __device__ __forceinline__ void join_store4(bf16* p, float4 v) {
  join_bf16x4 t;
  t.v[0] = from_float<bf16>(v.x);
  t.v[1] = from_float<bf16>(v.y);
  t.v[2] = from_float<bf16>(v.z);
  t.v[3] = from_float<bf16>(v.w);
  *reinterpret_cast<join_bf16x4*>(p) = t;
}
static __device__ __forceinline__ void fma4(float4& s, float f, const float4& y) {
  s.x = fmaf(f, y.x, s.x);
  s.y = fmaf(f, y.y, s.y);
  s.z = fmaf(f, y.z, s.z);
  s.w = fmaf(f, y.w, s.w);
}
static __device__ __forceinline__ float4 mul4(const float4& a, float f, const float4& b) {
  return float4{a.x * f * b.x, a.y * f * b.y, a.z * f * b.z, a.w * f * b.w};
}
static __device__ __forceinline__ float dot4(const float4& a) { return (a.x * a.x + a.y * a.y) + (a.z * a.z + a.w * a.w); }

// four elements of a term at `at`; a stack's parts are asked for four at a time and added in order
static __device__ __forceinline__ float4 term4(const JoinTerm& t, size_t at) {
  if (t.dtype == kBF16) return join_load4(static_cast<const bf16*>(t.y) + at);
  const float* y = static_cast<const float*>(t.y) + at;
  float4 s = join_load4(y);
  for (int p0 = 1; p0 < t.parts; p0 += 4) {
    float4 v[4];
#pragma unroll
    for (int p = 0; p < 4; ++p) v[p] = p0 + p < t.parts ? join_load4(y + (size_t)(p0 + p) * t.part_stride) : float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int p = 0; p < 4; ++p)
      if (p0 + p < t.parts) fma4(s, 1.f, v[p]);
  }
  return s;
}
static __device__ __forceinline__ float term1(const JoinTerm& t, size_t at) {
  if (t.dtype == kBF16) return to_float(static_cast<const bf16*>(t.y)[at]);
  const float* y = static_cast<const float*>(t.y) + at;
  float s = y[0];
  for (int p = 1; p < t.parts; ++p) s += y[(size_t)p * t.part_stride];
  return s;
}

// inv[g] = 1 / sqrt(mean over the row's part g of squares + eps) for `groups` equal parts of a multiple of 4 elements; a
// thread brings the sums of squares of its pieces of 4 elements.  The order of a part's sum is fixed by the sizes alone.
template <int NT, int MAXV>
static __device__ __forceinline__ void group_inverses(const float (&ss)[MAXV], int nvec, int groups, float eps, float* pieces, float* inv) {
  const int lane = threadIdx.x & (kWave - 1), per = nvec / groups;
  __syncthreads();                 // whoever reads `pieces` or `inv` of the norm before is done
#pragma unroll
  for (int v = 0; v < MAXV; ++v) {
    const int i = v * NT + threadIdx.x;
    if (i < nvec) pieces[i] = ss[v];
  }
  __syncthreads();
  for (int g = threadIdx.x / kWave; g < groups; g += NT / kWave) {
    float s = 0.f;
    for (int i = lane; i < per; i += kWave) s += pieces[g * per + i];
    s = wave_sum(s);
    if (lane == 0) inv[g] = rsqrtf(s / (float)(4 * per) + eps);
  }
  __syncthreads();
}

// Rows of a multiple of 4 elements, up to 4 NT MAXV: a thread keeps its pieces of the row (and of the normed terms) in
// registers.  NN: how many terms are normed.  GROUPED: some norm is made in groups (of a multiple of 4 elements).
template <typename TO, int NT, int MAXV, int NN, bool GROUPED>
__global__ __launch_bounds__(NT) void stream_join_vec_kernel(const JoinArgs A) {
  __shared__ float scratch[NT / kWave];
  __shared__ float pieces[GROUPED ? NT * MAXV : 1], ginv[GROUPED ? kJoinGroups : 1];
  const int r = blockIdx.x;
  const int row = A.rows ? A.rows[r] : r;
  const int H = A.H, nvec = H / 4;
  const size_t base = (size_t)row * H, obase = (size_t)r * H;
  float4 s[MAXV], y[NN > 0 ? NN : 1][MAXV];
  float ss[NN > 0 ? NN : 1];
#pragma unroll
  for (int n = 0; n < (NN > 0 ? NN : 1); ++n) ss[n] = 0.f;
#pragma unroll
  for (int v = 0; v < MAXV; ++v) {
    const int i = v * NT + threadIdx.x;
    s[v] = float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int n = 0; n < NN; ++n) y[n][v] = float4{0.f, 0.f, 0.f, 0.f};
    if (i < nvec) {
      if (A.x) s[v] = join_load4(A.x + base + 4 * i);
#pragma unroll
      for (int n = 0; n < NN; ++n) y[n][v] = term4(A.normed[n], base + 4 * i);
#pragma unroll
      for (int p = 0; p < kJoinPlain; ++p)
        if (p < A.n_plain) fma4(s[v], A.plain[p].factor, term4(A.plain[p], base + 4 * i));
    }
#pragma unroll
    for (int n = 0; n < NN; ++n) ss[n] += dot4(y[n][v]);
  }
#pragma unroll
  for (int n = 0; n < NN; ++n) {
    if constexpr (GROUPED) {
      float sq[MAXV];
#pragma unroll
      for (int v = 0; v < MAXV; ++v) sq[v] = dot4(y[n][v]);
      group_inverses<NT, MAXV>(sq, nvec, A.normed[n].groups, A.normed[n].eps, pieces, ginv);
      const int per = nvec / A.normed[n].groups;
#pragma unroll
      for (int v = 0; v < MAXV; ++v) {
        const int i = v * NT + threadIdx.x;
        if (i < nvec) fma4(s[v], A.normed[n].factor, mul4(y[n][v], ginv[i / per], join_load4(A.normed[n].w + 4 * i)));
      }
      continue;
    }
    const float inv = rsqrtf(block_sum<NT / kWave>(ss[n], scratch) / (float)H + A.normed[n].eps);
#pragma unroll
    for (int v = 0; v < MAXV; ++v) {
      const int i = v * NT + threadIdx.x;
      if (i < nvec) fma4(s[v], A.normed[n].factor, mul4(y[n][v], inv, join_load4(A.normed[n].w + 4 * i)));
    }
  }
  if (A.result || A.rounded) {
#pragma unroll
    for (int v = 0; v < MAXV; ++v) {
      const int i = v * NT + threadIdx.x;
      if (i >= nvec) continue;
      if (A.result) join_store4(A.result + obase + 4 * i, s[v]);
      if (A.rounded) join_store4(static_cast<TO*>(A.rounded) + obase + 4 * i, s[v]);
    }
  }
  if (A.first) {
#pragma unroll
    for (int v = 0; v < MAXV; ++v) {
      const int i = v * NT + threadIdx.x;
      if (i >= nvec) continue;
      const float4 f0 = join_load4(A.first + base + 4 * i);
      const float c0 = A.coef[0];
      float4 u = float4{c0 * f0.x, c0 * f0.y, c0 * f0.z, c0 * f0.w};
      const float* past = A.past + base + 4 * i;
      for (int j0 = 0; j0 < A.n_past; j0 += 8) {      // eight results asked for at once, added in order
        float4 p[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) p[j] = j0 + j < A.n_past ? join_load4(past + (size_t)(j0 + j) * A.past_stride) : float4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (j0 + j < A.n_past) fma4(u, A.coef[1 + j0 + j], p[j]);
      }
      fma4(u, A.coef[1 + A.n_past], s[v]);
      s[v] = u;
      if (A.xout) join_store4(A.xout + obase + 4 * i, u);
    }
  }
  if (A.n_norms == 0) return;
  if constexpr (GROUPED) {
    float sq[MAXV];
#pragma unroll
    for (int v = 0; v < MAXV; ++v) sq[v] = dot4(s[v]);
#pragma unroll
    for (int k = 0; k < kJoinNorms; ++k) {
      if (k >= A.n_norms) break;
      group_inverses<NT, MAXV>(sq, nvec, A.groups[k], A.eps[k], pieces, ginv);
      const int per = nvec / A.groups[k];
#pragma unroll
      for (int v = 0; v < MAXV; ++v) {
        const int i = v * NT + threadIdx.x;
        if (i < nvec) join_store4(static_cast<TO*>(A.h[k]) + obase + 4 * i, mul4(s[v], ginv[i / per], join_load4(A.w[k] + 4 * i)));
      }
    }
    return;
  }
  float us = 0.f;
#pragma unroll
  for (int v = 0; v < MAXV; ++v) us += dot4(s[v]);          // (pieces past the row's end are zeros)
  const float mean = block_sum<NT / kWave>(us, scratch) / (float)H;
#pragma unroll
  for (int k = 0; k < kJoinNorms; ++k) {
    if (k >= A.n_norms) break;
    const float inv = rsqrtf(mean + A.eps[k]);
#pragma unroll
    for (int v = 0; v < MAXV; ++v) {
      const int i = v * NT + threadIdx.x;
      if (i < nvec) join_store4(static_cast<TO*>(A.h[k]) + obase + 4 * i, mul4(s[v], inv, join_load4(A.w[k] + 4 * i)));
    }
  }
}

// Any width: the row's values are made again from the operands for every pass.
template <typename TO>
__global__ __launch_bounds__(256) void stream_join_kernel(const JoinArgs A) {
  __shared__ float scratch[4];
  __shared__ float inv[kJoinNormed][kJoinGroups], ninv[kJoinNorms][kJoinGroups];
  const int r = blockIdx.x;
  const int row = A.rows ? A.rows[r] : r;
  const int H = A.H;
  const size_t base = (size_t)row * H, obase = (size_t)r * H;
  int per[kJoinNormed], nper[kJoinNorms];
  for (int n = 0; n < kJoinNormed; ++n) {
    per[n] = H;
    if (n >= A.n_normed) continue;
    per[n] = H / A.normed[n].groups;
    for (int g = 0; g < A.normed[n].groups; ++g) {
      float ss = 0.f;
      for (int i = g * per[n] + threadIdx.x; i < (g + 1) * per[n]; i += 256) {
        const float v = term1(A.normed[n], base + i);
        ss = fmaf(v, v, ss);
      }
      const float f = rsqrtf(block_sum<4>(ss, scratch) / (float)per[n] + A.normed[n].eps);
      if (threadIdx.x == 0) inv[n][g] = f;
    }
  }
  __syncthreads();
  auto sum_at = [&](int i) {
    float s = A.x ? A.x[base + i] : 0.f;
    for (int p = 0; p < A.n_plain; ++p) s = fmaf(A.plain[p].factor, term1(A.plain[p], base + i), s);
    for (int n = 0; n < A.n_normed; ++n) s = fmaf(A.normed[n].factor, term1(A.normed[n], base + i) * inv[n][i / per[n]] * A.normed[n].w[i], s);
    return s;
  };
  auto average_at = [&](int i, float s) {
    if (!A.first) return s;
    float u = A.coef[0] * A.first[base + i];
    for (int j = 0; j < A.n_past; ++j) u = fmaf(A.coef[1 + j], A.past[(size_t)j * A.past_stride + base + i], u);
    return fmaf(A.coef[1 + A.n_past], s, u);
  };
  float us = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) {
    const float s = sum_at(i), u = average_at(i, s);
    us = fmaf(u, u, us);
    if (A.result) A.result[obase + i] = s;
    if (A.rounded) static_cast<TO*>(A.rounded)[obase + i] = from_float<TO>(s);
    if (A.xout && A.first) A.xout[obase + i] = u;
  }
  if (A.n_norms == 0) return;
  const float mean = block_sum<4>(us, scratch) / (float)H;
  for (int k = 0; k < A.n_norms; ++k) {
    nper[k] = H / A.groups[k];
    for (int g = 0; g < A.groups[k]; ++g) {
      float m = mean;
      if (A.groups[k] > 1) {
        float gs = 0.f;
        for (int i = g * nper[k] + threadIdx.x; i < (g + 1) * nper[k]; i += 256) {
          const float u = average_at(i, sum_at(i));
          gs = fmaf(u, u, gs);
        }
        m = block_sum<4>(gs, scratch) / (float)nper[k];
      }
      if (threadIdx.x == 0) ninv[k][g] = rsqrtf(m + A.eps[k]);
    }
  }
  __syncthreads();
  for (int i = threadIdx.x; i < H; i += 256) {
    const float u = average_at(i, sum_at(i));
    for (int k = 0; k < A.n_norms; ++k)
      static_cast<TO*>(A.h[k])[obase + i] = from_float<TO>(u * ninv[k][i / nper[k]] * A.w[k][i]);
  }
}

// out[t] = (x / sqrt(mean(x^2) + eps)) w, x = float(table[ids[t]]) * scale: an embedding that is normed.
template <typename T>
__global__ __launch_bounds__(256) void embed_norm_kernel(const T* __restrict__ table, const int* __restrict__ ids, float scale,
                                                         const float* __restrict__ w, float eps, float* __restrict__ out, int H) {
  __shared__ float scratch[4];
  const T* row = table + (size_t)ids[blockIdx.x] * H;
  float* o = out + (size_t)blockIdx.x * H;
  float ss = 0.f;
  for (int i = threadIdx.x; i < H; i += 256) {
    const float v = to_float(row[i]) * scale;
    ss = fmaf(v, v, ss);
  }
  const float inv = rsqrtf(block_sum<4>(ss, scratch) / (float)H + eps);
  for (int i = threadIdx.x; i < H; i += 256) o[i] = to_float(row[i]) * scale * inv * w[i];
}

// Rows of a multiple of 4 elements, up to 4 NT MAXV, kept in registers between the sum and the store.
template <typename T, int NT, int MAXV>
__global__ __launch_bounds__(NT) void embed_norm_vec_kernel(const T* __restrict__ table, const int* __restrict__ ids, float scale,
                                                            const float* __restrict__ w, float eps, float* __restrict__ out, int H) {
  __shared__ float scratch[NT / kWave];
  const T* row = table + (size_t)ids[blockIdx.x] * H;
  float* o = out + (size_t)blockIdx.x * H;
  const int nvec = H / 4;
  float4 x[MAXV];
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < MAXV; ++v) {
    const int i = v * NT + threadIdx.x;
    x[v] = i < nvec ? join_load4(row + 4 * i) : float4{0.f, 0.f, 0.f, 0.f};
    x[v] = float4{x[v].x * scale, x[v].y * scale, x[v].z * scale, x[v].w * scale};
    ss += dot4(x[v]);
  }
  const float inv = rsqrtf(block_sum<NT / kWave>(ss, scratch) / (float)H + eps);
#pragma unroll
  for (int v = 0; v < MAXV; ++v) {
    const int i = v * NT + threadIdx.x;
    if (i < nvec) join_store4(o + 4 * i, mul4(x[v], inv, join_load4(w + 4 * i)));
  }
}

template <typename TO>
static void launch_join(const JoinArgs& A, int n, hipStream_t stream, bool aligned) {
  const int H = A.H;
  bool grouped = false;
  for (int k = 0; k < A.n_normed; ++k) grouped = grouped || A.normed[k].groups > 1;
  for (int k = 0; k < A.n_norms; ++k) grouped = grouped || A.groups[k] > 1;
#define XI_JOIN_G(NT, MAXV, GR)                                                                          \
  do {                                                                                                   \
    if (A.n_normed == 0) stream_join_vec_kernel<TO, NT, MAXV, 0, GR><<<n, NT, 0, stream>>>(A);           \
    else if (A.n_normed == 1) stream_join_vec_kernel<TO, NT, MAXV, 1, GR><<<n, NT, 0, stream>>>(A);      \
    else stream_join_vec_kernel<TO, NT, MAXV, 2, GR><<<n, NT, 0, stream>>>(A);                           \
  } while (0)
#define XI_JOIN_N(NT, MAXV)                     \
  do {                                          \
    if (grouped) XI_JOIN_G(NT, MAXV, true);     \
    else XI_JOIN_G(NT, MAXV, false);            \
  } while (0)
  if (!aligned || H > 16384) {
    stream_join_kernel<TO><<<n, 256, 0, stream>>>(A);
  } else if (n <= 256 && H > 1024) {            // few rows: all of a row's loads in flight at once
    if (H <= 4096) XI_JOIN_N(1024, 1);
    else if (H <= 8192) XI_JOIN_N(1024, 2);
    else XI_JOIN_N(1024, 4);
  } else {
    if (H <= 1024) XI_JOIN_N(256, 1);
    else if (H <= 2048) XI_JOIN_N(256, 2);
    else if (H <= 4096) XI_JOIN_N(256, 4);
    else if (H <= 8192) XI_JOIN_N(512, 4);
    else XI_JOIN_N(1024, 4);
  }
#undef XI_JOIN_N
#undef XI_JOIN_G
}

}  // namespace xi

using namespace xi;

extern "C" {

// Terms in arrays of length n_terms: y[k] rows [*, H] in dtype[k] (a stack of parts[k] float32 partial sums part_stride
// elements apart if parts[k] > 1), weight[k] float32 [H] (null: a plain term), eps[k], factor[k], groups[k].  At most 3 plain and
// 2 normed.  norm_groups[k]: the groups of norm k.
// first float32 rows or null; past: n_past results past_stride elements apart; coef float32 [n_past + 2].
int xi_stream_join(const float* x, int n_terms, const void* const* y, const int* dtype, const int* parts, long long part_stride,
                   const float* const* weight, const float* eps, const float* factor, const int* groups, float* result, void* rounded,
                   const float* first, const float* past, long long past_stride, int n_past, const float* coef, float* xout,
                   int n_norms, const float* const* norm_w, const float* norm_eps, const int* norm_groups, void* const* norm_out, int out_dtype,
                   const int* rows, int n, int H, hipStream_t stream) {
  XI_CHECK(n >= 0 && H > 0 && n_terms >= 0 && n_norms >= 0 && n_norms <= kJoinNorms, "stream_join: bad sizes n=%d H=%d terms=%d norms=%d",
           n, H, n_terms, n_norms);
  XI_CHECK(out_dtype == kF32 || out_dtype == kBF16, "stream_join: unknown dtype %d", out_dtype);
  XI_CHECK(first == nullptr || (coef != nullptr && n_past >= 0 && (n_past == 0 || past != nullptr)), "stream_join: an average needs its results and weights");
  XI_CHECK(xout == nullptr || first != nullptr, "stream_join: the average's row without an average");
  if (n == 0) return 0;
  JoinArgs A{};
  bool aligned = H % 4 == 0;
  auto whole = [&](const void* p, size_t bytes) { aligned = aligned && (p == nullptr || reinterpret_cast<uintptr_t>(p) % bytes == 0); };
  const size_t ob = out_dtype == kF32 ? 16 : 8;
  A.x = x;
  whole(x, 16);
  for (int k = 0; k < n_terms; ++k) {
    XI_CHECK(y[k] && (dtype[k] == kF32 || dtype[k] == kBF16) && parts[k] >= 1 && (parts[k] == 1 || dtype[k] == kF32),
             "stream_join: term %d is no rows of a known type", k);
    JoinTerm t;
    t.y = y[k];
    t.part_stride = (size_t)part_stride;
    t.w = weight[k];
    t.parts = parts[k];
    t.dtype = dtype[k];
    t.eps = eps[k];
    t.factor = factor[k];
    whole(t.y, dtype[k] == kF32 ? 16 : 8);
    whole(t.w, 16);
    if (parts[k] > 1 && part_stride % 4) aligned = false;
    if (t.w) {
      t.groups = groups[k];
      XI_CHECK(t.groups >= 1 && t.groups <= kJoinGroups && H % t.groups == 0, "stream_join: rows of %d in %d groups", H, t.groups);
      if (t.groups > 1 && (H / t.groups) % 4) aligned = false;
      XI_CHECK(A.n_normed < kJoinNormed, "stream_join: more than %d normed terms", kJoinNormed);
      A.normed[A.n_normed++] = t;
    } else {
      XI_CHECK(A.n_plain < kJoinPlain, "stream_join: more than %d plain terms", kJoinPlain);
      A.plain[A.n_plain++] = t;
    }
  }
  A.result = result;
  A.rounded = rounded;
  A.first = first;
  A.past = past;
  A.past_stride = (size_t)past_stride;
  A.n_past = n_past;
  A.coef = coef;
  A.xout = xout;
  whole(result, 16);
  whole(rounded, ob);
  whole(first, 16);
  whole(past, 16);
  whole(xout, 16);
  if (past_stride % 4) aligned = false;
  A.n_norms = n_norms;
  for (int k = 0; k < n_norms; ++k) {
    XI_CHECK(norm_w[k] && norm_out[k], "stream_join: norm %d without a weight or a place", k);
    A.w[k] = norm_w[k];
    A.eps[k] = norm_eps[k];
    A.groups[k] = norm_groups[k];
    XI_CHECK(A.groups[k] >= 1 && A.groups[k] <= kJoinGroups && H % A.groups[k] == 0, "stream_join: rows of %d in %d groups", H, A.groups[k]);
    if (A.groups[k] > 1 && (H / A.groups[k]) % 4) aligned = false;
    A.h[k] = norm_out[k];
    whole(norm_w[k], 16);
    whole(norm_out[k], ob);
  }
  A.rows = rows;
  A.H = H;
  if (out_dtype == kF32) launch_join<float>(A, n, stream, aligned);
  else launch_join<bf16>(A, n, stream, aligned);
  XI_LAUNCH_CHECK("stream_join");
  return 0;
}

// table [V, H] in `dtype`, ids int32 [T], w float32 [H], out float32 [T, H].
int xi_embed_norm(const void* table, int dtype, const int* ids, float scale, const float* w, float eps, float* out, int n_tok, int H,
                  hipStream_t stream) {
  XI_CHECK(n_tok >= 0 && H > 0 && w, "embed_norm: bad sizes T=%d H=%d", n_tok, H);
  XI_CHECK(dtype == kF32 || dtype == kBF16, "embed_norm: unknown dtype %d", dtype);
  if (n_tok == 0) return 0;
  if (H % 4 == 0 && H <= 8192 && ((reinterpret_cast<uintptr_t>(table) | reinterpret_cast<uintptr_t>(w) | reinterpret_cast<uintptr_t>(out)) & 15) == 0) {
#define XI_EN(NT, MAXV)                                                                                                                  \
  do {                                                                                                                                   \
    if (dtype == kF32) embed_norm_vec_kernel<float, NT, MAXV><<<n_tok, NT, 0, stream>>>((const float*)table, ids, scale, w, eps, out, H); \
    else embed_norm_vec_kernel<bf16, NT, MAXV><<<n_tok, NT, 0, stream>>>((const bf16*)table, ids, scale, w, eps, out, H);                \
  } while (0)
    if (H <= 1024) XI_EN(256, 1);
    else if (n_tok <= 256) XI_EN(1024, 2);
    else if (H <= 4096) XI_EN(256, 4);
    else XI_EN(512, 4);
#undef XI_EN
    XI_LAUNCH_CHECK("embed_norm");
    return 0;
  }
  if (dtype == kF32) embed_norm_kernel<float><<<n_tok, 256, 0, stream>>>((const float*)table, ids, scale, w, eps, out, H);
  else embed_norm_kernel<bf16><<<n_tok, 256, 0, stream>>>((const bf16*)table, ids, scale, w, eps, out, H);
  XI_LAUNCH_CHECK("embed_norm");
  return 0;
}

}  // extern "C"
