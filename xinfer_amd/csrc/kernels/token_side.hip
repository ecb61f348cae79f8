// A layer's own input for the token: g[t, d] = gelu_tanh(z[t, d]) * e[ids[t], offset + d], z = W x, e a table row's part
// that belongs to the layer.  `side_mul_kernel` takes z as a product left it (rows, or a stack of float32 partial sums);
// `side_gate_kernel` makes z itself in steps of few tokens: a workgroup owns one output d, its waves a part of K each, and
// takes up to kSideTok tokens at a time, so that a row of W is read once for all of them.  Float32 until the one rounding of g.
#include "common.h"

namespace xi {

static __device__ __forceinline__ float side_gelu(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

template <typename T>
__global__ __launch_bounds__(256) void side_mul_kernel(const void* __restrict__ z, int z_f32, int parts, size_t part_stride,
                                                       const T* __restrict__ table, long long row_len, int offset,
                                                       const int* __restrict__ ids, T* __restrict__ out, int dim, long long total) {
  for (long long i = (long long)blockIdx.x * 256 + threadIdx.x; i < total; i += (long long)gridDim.x * 256) {
    const long long t = i / dim;
    const int d = (int)(i - t * dim);
    float v;
    if (z_f32) {
      const float* zp = static_cast<const float*>(z) + i;
      v = zp[0];
      for (int p = 1; p < parts; ++p) v += zp[(size_t)p * part_stride];
    } else {
      v = to_float(static_cast<const bf16*>(z)[i]);
    }
    out[i] = from_float<T>(side_gelu(v) * to_float(table[(size_t)ids[t] * row_len + offset + d]));
  }
}

constexpr int kSideTok = 8, kSideWaves = 4;

// K a multiple of 8, bfloat16
__global__ __launch_bounds__(kSideWaves* kWave) void side_gate_kernel(const bf16* __restrict__ x, const bf16* __restrict__ w,
                                                        const bf16* __restrict__ table, long long row_len, int offset,
                                                        const int* __restrict__ ids, bf16* __restrict__ out, int n_tok, int dim, int K) {
  __shared__ float part[kSideWaves][kSideTok];
  const int d = blockIdx.x, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int t0 = blockIdx.y * kSideTok;
  float acc[kSideTok];
#pragma unroll
  for (int t = 0; t < kSideTok; ++t) acc[t] = 0.f;
  for (int k = 8 * threadIdx.x; k < K; k += 8 * kSideWaves * kWave) {
    const uint4 wr = *reinterpret_cast<const uint4*>(w + (size_t)d * K + k);
    const unsigned wu[4] = {wr.x, wr.y, wr.z, wr.w};
    uint4 xr[kSideTok];
#pragma unroll
    for (int t = 0; t < kSideTok; ++t) {
      const int tt = t0 + t < n_tok ? t0 + t : n_tok - 1;
      xr[t] = *reinterpret_cast<const uint4*>(x + (size_t)tt * K + k);
    }
#pragma unroll
    for (int t = 0; t < kSideTok; ++t) {
      const unsigned xu[4] = {xr[t].x, xr[t].y, xr[t].z, xr[t].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        acc[t] = fmaf(__uint_as_float(wu[e] << 16), __uint_as_float(xu[e] << 16), acc[t]);
        acc[t] = fmaf(__uint_as_float(wu[e] & 0xffff0000u), __uint_as_float(xu[e] & 0xffff0000u), acc[t]);
      }
    }
  }
#pragma unroll
  for (int t = 0; t < kSideTok; ++t) {
    const float z = wave_sum(acc[t]);
    if (lane == 0) part[wave][t] = z;
  }
  __syncthreads();
  const int t = threadIdx.x;
  if (t < kSideTok && t0 + t < n_tok) {
    const float z = (part[0][t] + part[1][t]) + (part[2][t] + part[3][t]);
    out[(size_t)(t0 + t) * dim + d] = from_float<bf16>(side_gelu(z) * to_float(table[(size_t)ids[t0 + t] * row_len + offset + d]));
  }
}

}  // namespace xi

using namespace xi;

extern "C" {

// z [T, dim] in z_dtype (a stack of `parts` float32 partial sums part_stride elements apart if parts > 1); table rows of
// row_len elements in `dtype`, the layer's part from `offset`; ids int32 [T]; out [T, dim] in `dtype`.
int xi_side_mul(const void* z, int z_dtype, int parts, long long part_stride, const void* table, long long row_len, int offset,
                const int* ids, void* out, int dtype, int n_tok, int dim, hipStream_t stream) {
  XI_CHECK(n_tok >= 0 && dim > 0 && offset >= 0 && row_len >= (long long)offset + dim, "side_mul: bad sizes T=%d dim=%d offset=%d", n_tok, dim, offset);
  XI_CHECK((z_dtype == kF32 || z_dtype == kBF16) && parts >= 1 && (parts == 1 || z_dtype == kF32), "side_mul: the gate's rows are of no known form");
  if (n_tok == 0) return 0;
  const long long total = (long long)n_tok * dim;
  const long long want = (total + 255) / 256;
  const unsigned grid = (unsigned)(want < 65536 ? want : 65536);
  if (dtype == kF32)
    side_mul_kernel<float><<<grid, 256, 0, stream>>>(z, z_dtype == kF32, parts, (size_t)part_stride, (const float*)table, row_len,
                                                     offset, ids, (float*)out, dim, total);
  else if (dtype == kBF16)
    side_mul_kernel<bf16><<<grid, 256, 0, stream>>>(z, z_dtype == kF32, parts, (size_t)part_stride, (const bf16*)table, row_len,
                                                    offset, ids, (bf16*)out, dim, total);
  else XI_CHECK(false, "side_mul: unknown dtype %d", dtype);
  XI_LAUNCH_CHECK("side_mul");
  return 0;
}

// bfloat16: x [T, K], w [dim, K], K a multiple of 8; table, ids, out as above.
int xi_side_gate(const void* x, const void* w, const void* table, long long row_len, int offset, const int* ids, void* out, int n_tok,
                 int dim, int K, hipStream_t stream) {
  XI_CHECK(n_tok >= 0 && dim > 0 && K > 0 && K % 8 == 0 && offset >= 0 && row_len >= (long long)offset + dim,
           "side_gate: bad sizes T=%d dim=%d K=%d offset=%d", n_tok, dim, K, offset);
  XI_CHECK((reinterpret_cast<uintptr_t>(x) & 15) == 0 && (reinterpret_cast<uintptr_t>(w) & 15) == 0, "side_gate: rows in whole 16-byte chunks");
  if (n_tok == 0) return 0;
  dim3 grid((unsigned)dim, (unsigned)((n_tok + kSideTok - 1) / kSideTok));
  XI_CHECK(grid.y <= 65535u, "side_gate: too many tokens");
  side_gate_kernel<<<grid, kSideWaves * kWave, 0, stream>>>((const bf16*)x, (const bf16*)w, (const bf16*)table, row_len, offset, ids, (bf16*)out, n_tok,
                                             dim, K);
  XI_LAUNCH_CHECK("side_gate");
  return 0;
}

}  // extern "C"
