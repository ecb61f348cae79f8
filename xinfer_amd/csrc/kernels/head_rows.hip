// A packed projection row [q (nq d) | k (nkv d) | v (nkv dv)] made ready for attention head by head, one wave a
// (token, head):  a bias per column of the row (`bias`, or none) is added, a q or k head is divided by its root mean
// square over d and multiplied by a weight [d] that the q (or k) heads share (`qw`, `kw`, or none), its first `rot` dims
// turn by the token's position (pairs (2i, 2i + 1) if interleaved, else (i, i + rot / 2); float32 tables [positions,
// rot / 2]), and then, with `unit`, it is divided by its root mean square over d without a weight (eps inside the root
// both times).  q goes to q_out [T, nq, d], k and v into the paged cache at `slots` (a negative slot stores nothing).  K
// pool [pages, nkv, page, d]; V pool [pages, nkv, page, dv] or, grouped, [pages, nkv, page / 8, dv, 8].  The value head size may differ from d.
// The rows may be longer than that (`row_stride`), and the values' first column is `v_col`: behind the keys, or the keys'
// own columns (values that are the keys as projected, before norm and rotation).  With `vcos` / `vsin` (float32 [positions,
// dv / 2]) a value head turns by its position over all its dims, in the keys' layout of pairs, and is cached so.
// Everything between the read and the one rounding of the store is float32.
//
// `head_finish_kernel`: what follows such an attention, in place on its result [T, H, dv]: every head turns back by its own
// position (the same tables, the angle negated), and every element is multiplied by sigmoid(gate) (columns of a packed row).
#include "common.h"

namespace xi {

constexpr int kHeadRowWaves = 4;
constexpr int kHeadRowMost = 1024;      // longest head

template <typename T>
__global__ __launch_bounds__(kHeadRowWaves* kWave) void head_rows_kernel(
    const T* __restrict__ qkv, const long long* __restrict__ slots, T* __restrict__ q_out, T* __restrict__ k_cache,
    T* __restrict__ v_cache, int page_size, long long pairs, int nq, int nkv, int d, int dv, int v_grouped,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, int rot, int interleaved,
    const int* __restrict__ positions, int unit, float eps, const float* __restrict__ bias, const float* __restrict__ qw,
    const float* __restrict__ kw, long long row_stride, int v_col, const float* __restrict__ vcos, const float* __restrict__ vsin) {
  extern __shared__ float head_s[];                // [waves][d]
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const long long pair = (long long)blockIdx.x * kHeadRowWaves + wave;
  if (pair >= pairs) return;
  const int heads = nq + 2 * nkv;
  const long long t = pair / heads;
  const int h = (int)(pair - t * heads);
  const T* row = qkv + (size_t)t * row_stride;
  const long long slot = slots[t];
  const size_t page = slot < 0 ? 0 : (size_t)(slot / page_size);
  const int off = slot < 0 ? 0 : (int)(slot % page_size);
  if (h >= nq + nkv) {                             // a value head: a copy, or turned by its position
    if (slot < 0) return;
    const int hv = h - nq - nkv;
    const T* src = row + v_col + (size_t)hv * dv;
    const float* vb = bias ? bias + v_col + (size_t)hv * dv : nullptr;
    const size_t base = (page * nkv + hv) * (size_t)page_size * dv;
    auto place = [&](int c) {
      return v_grouped ? base + ((size_t)(off >> 3) * dv + c) * 8 + (off & 7) : base + (size_t)off * dv + c;
    };
    if (vcos) {
      const int vhalf = dv / 2;
      const size_t vrow = (size_t)positions[t] * vhalf;
      for (int i = lane; i < vhalf; i += kWave) {
        const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + vhalf;
        const float a = to_float(src[ia]) + (vb ? vb[ia] : 0.f), b = to_float(src[ib]) + (vb ? vb[ib] : 0.f);
        const float cs = vcos[vrow + i], sn = vsin[vrow + i];
        v_cache[place(ia)] = from_float<T>(a * cs - b * sn);
        v_cache[place(ib)] = from_float<T>(b * cs + a * sn);
      }
      return;
    }
    for (int c = lane; c < dv; c += kWave) v_cache[place(c)] = vb ? from_float<T>(to_float(src[c]) + vb[c]) : src[c];
    return;
  }
  const bool is_q = h < nq;
  if (!is_q && slot < 0) return;
  const T* src = row + (size_t)h * d;              // k heads follow the q heads
  float* x = head_s + (size_t)wave * d;
  const int half = rot / 2;
  const size_t trow = rot ? (size_t)positions[t] * half : 0;
  float ss = 0.f;
  const float* wt = is_q ? qw : kw;
  const float* hb = bias ? bias + (size_t)h * d : nullptr;
  for (int i = lane; i < half; i += kWave) {
    const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + half;
    const float a = to_float(src[ia]) + (hb ? hb[ia] : 0.f), b = to_float(src[ib]) + (hb ? hb[ib] : 0.f);
    x[ia] = a;
    x[ib] = b;
    ss = fmaf(a, a, fmaf(b, b, ss));
  }
  for (int i = rot + lane; i < d; i += kWave) {
    const float a = to_float(src[i]) + (hb ? hb[i] : 0.f);
    x[i] = a;
    ss = fmaf(a, a, ss);
  }
  const float before = wt ? rsqrtf(wave_sum(ss) / (float)d + eps) : 1.f;
  ss = 0.f;
  // (a lane reads back what it wrote itself: pairs and single dims are dealt out the same way in every loop)
  for (int i = lane; i < half; i += kWave) {
    const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + half;
    const float a = wt ? x[ia] * before * wt[ia] : x[ia], b = wt ? x[ib] * before * wt[ib] : x[ib];
    const float cs = cos_t[trow + i], sn = sin_t[trow + i];
    const float ra = a * cs - b * sn, rb = b * cs + a * sn;
    x[ia] = ra;
    x[ib] = rb;
    ss = fmaf(ra, ra, fmaf(rb, rb, ss));
  }
  for (int i = rot + lane; i < d; i += kWave) {
    const float a = wt ? x[i] * before * wt[i] : x[i];
    x[i] = a;
    ss = fmaf(a, a, ss);
  }
  const float inv = unit ? rsqrtf(wave_sum(ss) / (float)d + eps) : 1.f;
  __builtin_amdgcn_wave_barrier();
  T* dst = is_q ? q_out + ((size_t)t * nq + h) * d : k_cache + ((page * nkv + (h - nq)) * (size_t)page_size + off) * d;
  for (int i = lane; i < half; i += kWave) {
    const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + half;
    dst[ia] = from_float<T>(x[ia] * inv);
    dst[ib] = from_float<T>(x[ib] * inv);
  }
  for (int i = rot + lane; i < d; i += kWave) dst[i] = from_float<T>(x[i] * inv);
}

// One thread: a pair of dims (turned) or one dim (not turned) of a token's head.
template <typename T>
__global__ __launch_bounds__(256) void head_finish_kernel(T* __restrict__ x, const T* __restrict__ gate, long long gate_stride,
                                                          const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                                          const int* __restrict__ positions, int interleaved, int H, int dv,
                                                          long long units) {
  const long long u = (long long)blockIdx.x * 256 + threadIdx.x;
  if (u >= units) return;
  const int width = H * dv;
  if (!cos_t) {
    const long long t = u / width;
    const int i = (int)(u - t * width);
    const float g = to_float(gate[t * gate_stride + i]);
    x[u] = from_float<T>(to_float(x[u]) / (1.f + expf(-g)));
    return;
  }
  const int half = dv / 2, per = H * half;
  const long long t = u / per;
  const int r = (int)(u - t * per), h = r / half, i = r - h * half;
  const int ia = h * dv + (interleaved ? 2 * i : i), ib = h * dv + (interleaved ? 2 * i + 1 : i + half);
  T* row = x + (size_t)t * width;
  const float a = to_float(row[ia]), b = to_float(row[ib]);
  const float cs = cos_t[(size_t)positions[t] * half + i], sn = sin_t[(size_t)positions[t] * half + i];
  float oa = a * cs + b * sn, ob = b * cs - a * sn;
  if (gate) {
    oa /= 1.f + expf(-to_float(gate[t * gate_stride + ia]));
    ob /= 1.f + expf(-to_float(gate[t * gate_stride + ib]));
  }
  row[ia] = from_float<T>(oa);
  row[ib] = from_float<T>(ob);
}

// bfloat16 in whole chunks of 8: a thread takes 8 dims, or (turned) 8 dims and their 8 partners half a head further on.
struct alignas(16) head_bf8 { bf16 v[8]; };
static __device__ __forceinline__ float fast_sigmoid_over(float v, float g) { return v / (1.f + __expf(-g)); }
template <bool TURN, bool GATE>
__global__ __launch_bounds__(256) void head_finish_vec_kernel(bf16* __restrict__ x, const bf16* __restrict__ gate, long long gate_stride,
                                                              const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                                              const int* __restrict__ positions, int H, int dv, long long units) {
  const long long u = (long long)blockIdx.x * 256 + threadIdx.x;
  if (u >= units) return;
  const int width = H * dv;
  if constexpr (!TURN) {
    const int per = width / 8;
    const long long t = u / per;
    const int i = 8 * (int)(u - t * per);
    head_bf8 a = *reinterpret_cast<const head_bf8*>(x + (size_t)t * width + i);
    const head_bf8 g = *reinterpret_cast<const head_bf8*>(gate + t * gate_stride + i);
#pragma unroll
    for (int e = 0; e < 8; ++e) a.v[e] = from_float<bf16>(fast_sigmoid_over(to_float(a.v[e]), to_float(g.v[e])));
    *reinterpret_cast<head_bf8*>(x + (size_t)t * width + i) = a;
  } else {
    const int half = dv / 2, ph = half / 8, per = H * ph;
    const long long t = u / per;
    const int r = (int)(u - t * per), h = r / ph, i = 8 * (r - h * ph);
    const int ia = h * dv + i, ib = ia + half;
    bf16* row = x + (size_t)t * width;
    head_bf8 a = *reinterpret_cast<const head_bf8*>(row + ia), b = *reinterpret_cast<const head_bf8*>(row + ib);
    head_bf8 ga, gb;
    if constexpr (GATE) {
      ga = *reinterpret_cast<const head_bf8*>(gate + t * gate_stride + ia);
      gb = *reinterpret_cast<const head_bf8*>(gate + t * gate_stride + ib);
    }
    const size_t at = (size_t)positions[t] * half + i;
    float cs[8], sn[8];
#pragma unroll
    for (int e = 0; e < 8; e += 4) {
      const float4 c4 = *reinterpret_cast<const float4*>(cos_t + at + e), s4 = *reinterpret_cast<const float4*>(sin_t + at + e);
      cs[e] = c4.x; cs[e + 1] = c4.y; cs[e + 2] = c4.z; cs[e + 3] = c4.w;
      sn[e] = s4.x; sn[e + 1] = s4.y; sn[e + 2] = s4.z; sn[e + 3] = s4.w;
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float av = to_float(a.v[e]), bv = to_float(b.v[e]);
      float oa = av * cs[e] + bv * sn[e], ob = bv * cs[e] - av * sn[e];
      if constexpr (GATE) {
        oa = fast_sigmoid_over(oa, to_float(ga.v[e]));
        ob = fast_sigmoid_over(ob, to_float(gb.v[e]));
      }
      a.v[e] = from_float<bf16>(oa);
      b.v[e] = from_float<bf16>(ob);
    }
    *reinterpret_cast<head_bf8*>(row + ia) = a;
    *reinterpret_cast<head_bf8*>(row + ib) = b;
  }
}

}  // namespace xi

using namespace xi;

// x [T, H * dv] in `dtype`, changed in place.  gate: rows of gate_stride elements with H * dv columns from the given pointer, in
// `dtype` (null: none); cos_t / sin_t float32 [positions, dv / 2] (null: nothing turns); positions int32 [T].
extern "C" int xi_head_finish(void* x, int dtype, const void* gate, long long gate_stride, const float* cos_t, const float* sin_t,
                              const int* positions, int interleaved, int n_tok, int H, int dv, hipStream_t stream) {
  XI_CHECK(n_tok >= 0 && H > 0 && dv > 0, "head_finish: bad sizes T=%d H=%d dv=%d", n_tok, H, dv);
  XI_CHECK((gate == nullptr || gate_stride >= (long long)H * dv) && (gate || cos_t), "head_finish: nothing to do, or short gate rows");
  XI_CHECK((cos_t == nullptr) == (sin_t == nullptr) && (cos_t == nullptr || (positions && dv % 2 == 0)),
           "head_finish: heads of %d turn in pairs, by tables and positions", dv);
  XI_CHECK(dtype == kF32 || dtype == kBF16, "head_finish: unknown dtype %d", dtype);
  if (n_tok == 0) return 0;
  auto whole = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  const bool vec = dtype == kBF16 && whole(x) && whole(gate) && gate_stride % 8 == 0 && dv % (cos_t ? 16 : 8) == 0 &&
                   !(cos_t && interleaved) && whole(cos_t) && whole(sin_t);
  const long long units = (long long)n_tok * H * (cos_t ? dv / 2 : dv) / (vec ? 8 : 1);
  const long long blocks = (units + 255) / 256;
  XI_CHECK(blocks < (1ll << 31), "head_finish: too many tokens");
  if (vec) {
#define XI_HF(TURN, GATE)                                                                                                     \
  head_finish_vec_kernel<TURN, GATE><<<(unsigned)blocks, 256, 0, stream>>>((bf16*)x, (const bf16*)gate, gate_stride, cos_t, sin_t, \
                                                                           positions, H, dv, units)
    if (cos_t && gate) XI_HF(true, true);
    else if (cos_t) XI_HF(true, false);
    else XI_HF(false, true);
#undef XI_HF
  } else if (dtype == kF32) {
    head_finish_kernel<float><<<(unsigned)blocks, 256, 0, stream>>>((float*)x, (const float*)gate, gate_stride, cos_t, sin_t, positions,
                                                                    interleaved, H, dv, units);
  } else {
    head_finish_kernel<bf16><<<(unsigned)blocks, 256, 0, stream>>>((bf16*)x, (const bf16*)gate, gate_stride, cos_t, sin_t, positions,
                                                                   interleaved, H, dv, units);
  }
  XI_LAUNCH_CHECK("head_finish");
  return 0;
}

extern "C" int xi_head_rows(const void* qkv, int dtype, const long long* slots, void* q_out, void* k_cache, void* v_cache,
                            int page_size, int n_tok, int nq, int nkv, int d, int dv, int v_grouped, const float* cos_t,
                            const float* sin_t, int rot, int interleaved, const int* positions, int unit, float eps, const float* bias,
                            const float* qw, const float* kw, long long row_stride, int v_col, const float* vcos, const float* vsin,
                            hipStream_t stream) {
  XI_CHECK(v_col >= 0 && row_stride >= v_col + (long long)nkv * dv && row_stride >= (long long)(nq + nkv) * d,
           "head_rows: rows of %lld do not hold the heads", row_stride);
  XI_CHECK((vcos == nullptr) == (vsin == nullptr) && (vcos == nullptr || (positions && dv % 2 == 0)),
           "head_rows: value heads of %d turn in pairs, by tables and positions", dv);
  XI_CHECK(n_tok >= 0 && nq > 0 && nkv > 0 && d > 0 && dv > 0 && page_size > 0,
           "head_rows: bad sizes T=%d nq=%d nkv=%d d=%d dv=%d page=%d", n_tok, nq, nkv, d, dv, page_size);
  XI_CHECK(d <= kHeadRowMost, "head_rows: heads of up to %d dims, not %d", kHeadRowMost, d);
  XI_CHECK(rot >= 0 && rot % 2 == 0 && rot <= d, "head_rows: %d rotated dims of a head of %d", rot, d);
  XI_CHECK(rot == 0 || (cos_t && sin_t && positions), "head_rows: a rotation needs its tables and the positions");
  XI_CHECK(!v_grouped || page_size % 8 == 0, "head_rows: V in groups of eight keys needs pages of a multiple of 8 tokens, not %d",
           page_size);
  if (n_tok == 0) return 0;
  const long long pairs = (long long)n_tok * (nq + 2 * nkv);
  const long long blocks = (pairs + kHeadRowWaves - 1) / kHeadRowWaves;
  XI_CHECK(blocks < (1ll << 31), "head_rows: too many tokens");
  const size_t lds = (size_t)kHeadRowWaves * d * sizeof(float);
  if (dtype == kF32)
    head_rows_kernel<float><<<(unsigned)blocks, kHeadRowWaves * kWave, lds, stream>>>(
        (const float*)qkv, slots, (float*)q_out, (float*)k_cache, (float*)v_cache, page_size, pairs, nq, nkv, d, dv, v_grouped,
        cos_t, sin_t, rot, interleaved, positions, unit, eps, bias, qw, kw, row_stride, v_col, vcos, vsin);
  else if (dtype == kBF16)
    head_rows_kernel<bf16><<<(unsigned)blocks, kHeadRowWaves * kWave, lds, stream>>>(
        (const bf16*)qkv, slots, (bf16*)q_out, (bf16*)k_cache, (bf16*)v_cache, page_size, pairs, nq, nkv, d, dv, v_grouped, cos_t,
        sin_t, rot, interleaved, positions, unit, eps, bias, qw, kw, row_stride, v_col, vcos, vsin);
  else
    XI_CHECK(false, "head_rows: unknown dtype %d", dtype);
  XI_LAUNCH_CHECK("head_rows");
  return 0;
}
