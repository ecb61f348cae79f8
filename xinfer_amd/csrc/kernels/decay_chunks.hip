// Linear attention with one constant decay a head (S <- a S + k v^T, o = S^T q; optionally q, k, v behind silu) over long
// portions in bfloat16, on the matrix cores.  A portion is cut into chunks of up to 64 tokens; with S_c the state before a
// chunk of n tokens and i, j its tokens,
//
//   (1) its share          U = sum_j a^(n - 1 - j) k_j v_j^T
//   (2) the states         S_(c + 1) = a^n S_c + U, element by element from the request's slot, the last one back into it
//   (3) the results        o_i = a^(i + 1) q_i S_c + sum_(j <= i) a^(i - j) (q_i . k_j) v_j
//
// q, k and v enter as bfloat16 (behind silu: rounded once).  What is float32 in the walk token by token and would lose bits
// here (the decayed keys of (1), S_c and the decayed scores of (3)) is split into a bfloat16 and the bfloat16 of what is
// left, two products instead of one; sums are float32.  Factors a^n are exp2(n log2 a).
#include "common.h"

namespace xi {

typedef __attribute__((ext_vector_type(8))) __bf16 dc_bf16x8;
typedef __attribute__((ext_vector_type(4))) float dc_f32x4;

constexpr int kDcTok = 64;          // tokens of a chunk at most
constexpr int kDcCols = 128;        // value columns of a workgroup: 32 a wave
constexpr int kDcPad = 8;           // bf16 of padding a row in LDS
constexpr int kDcRow = kDcTok + kDcPad;

static __device__ __forceinline__ float dc_pow(float log2a, int n) { return n == 0 ? 1.f : exp2f((float)n * log2a); }
static __device__ __forceinline__ float dc_act(float x, int act) {
  return act ? x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x)) : x;
}
static __device__ __forceinline__ void dc_load8(const bf16* p, float (&v)[8]) {
  const uint4 a = *reinterpret_cast<const uint4*>(p);
  const unsigned u[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    v[2 * i] = __uint_as_float(u[i] << 16);
    v[2 * i + 1] = __uint_as_float(u[i] & 0xffff0000u);
  }
}
static __device__ __forceinline__ dc_bf16x8 dc_ld(const __bf16* p) { return *reinterpret_cast<const dc_bf16x8*>(p); }

struct DcArgs {
  const bf16 *q, *k, *v;
  long long q_stride, k_stride, v_stride;
  const float* decay;
  const int* first;                 // a chunk's tokens: first .. last - 1
  const int* last;
  float* shares;                    // float32 [chunks, H, dk, dv]
  const float* begins;              // float32 [chunks, H, dk, dv]
  float* out;                       // float32 [T, H, dv]
  int H, dk, dv, act;
  float q_scale, k_scale;
};

// (1) a workgroup of four waves: one chunk, one head, kDcCols value columns; wave w all key channels by its 32 columns.
// DKT: key channels in tiles of 16 (the tiles past dk multiply zeros and are not stored).
template <int DKT>
__global__ __launch_bounds__(256) void decay_share_kernel(const DcArgs A) {
  extern __shared__ __align__(16) unsigned char dc_smem[];
  __bf16* kh = reinterpret_cast<__bf16*>(dc_smem);                  // [16 DKT][kDcRow]: decayed keys, a channel a row
  __bf16* kl = kh + 16 * DKT * kDcRow;                              // what their rounding left
  __bf16* vt = kl + 16 * DKT * kDcRow;                              // [kDcCols][kDcRow]: values, a column a row
  const int c = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * kDcCols;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, j = lane >> 4;
  const int t0 = A.first[c], n = A.last[c] - t0;
  if (n <= 0) return;
  const float l2 = log2f(A.decay[h]);
  // a thread takes 8 channels of a token; consecutive threads take consecutive tokens, so that a wave's 2-byte stores of
  // one channel lie side by side
  const int tok = lane;
  const float wk = tok < n ? dc_pow(l2, n - 1 - tok) * A.k_scale : 0.f;
  for (int ch = 8 * wave; ch < 16 * DKT; ch += 32) {
    float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (tok < n && ch < A.dk) dc_load8(A.k + (size_t)(t0 + tok) * A.k_stride + (size_t)h * A.dk + ch, x);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float y = (float)(__bf16)dc_act(x[e], A.act) * wk;
      const __bf16 hi = (__bf16)y;
      kh[(ch + e) * kDcRow + tok] = hi;
      kl[(ch + e) * kDcRow + tok] = (__bf16)(y - (float)hi);
    }
  }
  for (int cc = 8 * wave; cc < kDcCols; cc += 32) {
    float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (tok < n && col0 + cc < A.dv) dc_load8(A.v + (size_t)(t0 + tok) * A.v_stride + (size_t)h * A.dv + col0 + cc, x);
#pragma unroll
    for (int e = 0; e < 8; ++e) vt[(cc + e) * kDcRow + tok] = (__bf16)dc_act(x[e], A.act);
  }
  __syncthreads();
  if (col0 + 32 * wave >= A.dv) return;
  dc_f32x4 acc[DKT][2];
#pragma unroll
  for (int a = 0; a < DKT; ++a)
#pragma unroll
    for (int b = 0; b < 2; ++b) acc[a][b] = dc_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < kDcTok / 32; ++s) {
    if (32 * s >= n) break;
    dc_bf16x8 vb[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) vb[b] = dc_ld(vt + (32 * wave + 16 * b + r) * kDcRow + 32 * s + 8 * j);
#pragma unroll
    for (int a = 0; a < DKT; ++a) {
      const dc_bf16x8 hi = dc_ld(kh + (16 * a + r) * kDcRow + 32 * s + 8 * j);
      const dc_bf16x8 lo = dc_ld(kl + (16 * a + r) * kDcRow + 32 * s + 8 * j);
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, vb[b], acc[a][b], 0, 0, 0);
        acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, vb[b], acc[a][b], 0, 0, 0);
      }
    }
  }
  // a lane's 4 values of a tile: channels 16 a + 4 j .. + 3, column 16 b + r
  float* U = A.shares + ((size_t)c * A.H + h) * A.dk * A.dv;
#pragma unroll
  for (int a = 0; a < DKT; ++a)
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const int col = col0 + 32 * wave + 16 * b + r;
      if (col >= A.dv) continue;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int ch = 16 * a + 4 * j + i;
        if (ch < A.dk) U[(size_t)ch * A.dv + col] = acc[a][b][i];
      }
    }
}

// (2) one thread an element of the state, one grid row a portion; a chunk's share makes room for the state before it.
__global__ __launch_bounds__(256) void decay_carry_kernel(float* __restrict__ state, long long slot_stride,
                                                          const long long* __restrict__ slots, const int* __restrict__ c0,
                                                          const int* __restrict__ count, const int* __restrict__ first,
                                                          const int* __restrict__ last, const float* __restrict__ decay,
                                                          float* __restrict__ shares, int H, int dk, int dv) {
  const int p = blockIdx.y;
  const size_t per = (size_t)H * dk * dv;
  const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= per) return;
  const float l2 = log2f(decay[e / ((size_t)dk * dv)]);
  float* slot = state + (size_t)slots[p] * slot_stride + e;
  float s = *slot;
  const int a = c0[p], b = a + count[p];
  for (int c4 = a; c4 < b; c4 += 4) {            // four shares asked for at once
    float u[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) u[k] = shares[(size_t)(c4 + k < b ? c4 + k : b - 1) * per + e];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (c4 + k >= b) break;
      shares[(size_t)(c4 + k) * per + e] = s;
      s = fmaf(dc_pow(l2, last[c4 + k] - first[c4 + k]), s, u[k]);
    }
  }
  *slot = s;
}

// (3) a workgroup of four waves: one chunk, one head, kDcCols value columns.  The scores are made by rows (wave w: tokens
// 16 w .. + 15), everything after by columns (wave w: its 32 value columns, all tokens).
template <int DKS>      // key channels in steps of 32
__global__ __launch_bounds__(256) void decay_result_kernel(const DcArgs A) {
  extern __shared__ __align__(16) unsigned char dc_smem[];
  constexpr int qrow = 32 * DKS + kDcPad;
  __bf16* qs = reinterpret_cast<__bf16*>(dc_smem);                  // [64][qrow]
  __bf16* ks = qs + kDcTok * qrow;                                  // [64][qrow]
  __bf16* vt = ks + kDcTok * qrow;                                  // [kDcCols][kDcRow]
  __bf16* ph = vt + kDcCols * kDcRow;                               // [64][kDcRow]: decayed scores
  __bf16* pl = ph + kDcTok * kDcRow;                                // what their rounding left
  const int c = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * kDcCols;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, j = lane >> 4;
  const int t0 = A.first[c], n = A.last[c] - t0;
  if (n <= 0) return;
  const float l2 = log2f(A.decay[h]);
  constexpr int CH = 4 * DKS;                                       // 16-byte chunks a row
  for (int i = tid; i < kDcTok * CH; i += 256) {
    const int tok = i / CH, ch = 8 * (i - tok * CH);
    float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, y[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (tok < n && ch < A.dk) {
      dc_load8(A.q + (size_t)(t0 + tok) * A.q_stride + (size_t)h * A.dk + ch, x);
      dc_load8(A.k + (size_t)(t0 + tok) * A.k_stride + (size_t)h * A.dk + ch, y);
    }
    dc_bf16x8 qb, kb;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      qb[e] = (__bf16)dc_act(x[e], A.act);
      kb[e] = (__bf16)dc_act(y[e], A.act);
    }
    *reinterpret_cast<dc_bf16x8*>(qs + tok * qrow + ch) = qb;
    *reinterpret_cast<dc_bf16x8*>(ks + tok * qrow + ch) = kb;
  }
  for (int cc = 8 * wave; cc < kDcCols; cc += 32) {
    float x[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (lane < n && col0 + cc < A.dv) dc_load8(A.v + (size_t)(t0 + lane) * A.v_stride + (size_t)h * A.dv + col0 + cc, x);
#pragma unroll
    for (int e = 0; e < 8; ++e) vt[(cc + e) * kDcRow + lane] = (__bf16)dc_act(x[e], A.act);
  }
  __syncthreads();
  {
    dc_f32x4 s[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) s[b] = dc_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < DKS; ++st) {
      const dc_bf16x8 qa = dc_ld(qs + (16 * wave + r) * qrow + 32 * st + 8 * j);
#pragma unroll
      for (int b = 0; b < 4; ++b)
        s[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa, dc_ld(ks + (16 * b + r) * qrow + 32 * st + 8 * j), s[b], 0, 0, 0);
    }
    // a lane's 4 values of tile b: queries 16 wave + 4 j + i, key 16 b + r
    const float scale = A.q_scale * A.k_scale;
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int qi = 16 * wave + 4 * j + i, kj = 16 * b + r;
        const float p = kj <= qi ? s[b][i] * scale * dc_pow(l2, qi - kj) : 0.f;
        const __bf16 hi = (__bf16)p;
        ph[qi * kDcRow + kj] = hi;
        pl[qi * kDcRow + kj] = (__bf16)(p - (float)hi);
      }
  }
  __syncthreads();
  const int wcol = col0 + 32 * wave;
  if (wcol >= A.dv) return;
  dc_f32x4 acc[4][2];
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (int b = 0; b < 2; ++b) acc[a][b] = dc_f32x4{0.f, 0.f, 0.f, 0.f};
  // q S_c: a lane reads 8 channels of one column of the state
  const float* S = A.begins + ((size_t)c * A.H + h) * A.dk * A.dv;
#pragma unroll
  for (int st = 0; st < DKS; ++st) {
    dc_bf16x8 sh[2], sl[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const int col = wcol + 16 * b + r;
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int ch = 32 * st + 8 * j + e;
        x[e] = (ch < A.dk && col < A.dv) ? S[(size_t)ch * A.dv + col] : 0.f;
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        sh[b][e] = (__bf16)x[e];
        sl[b][e] = (__bf16)(x[e] - (float)sh[b][e]);
      }
    }
#pragma unroll
    for (int a = 0; a < 4; ++a) {
      const dc_bf16x8 qa = dc_ld(qs + (16 * a + r) * qrow + 32 * st + 8 * j);
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa, sl[b], acc[a][b], 0, 0, 0);
        acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa, sh[b], acc[a][b], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float f = dc_pow(l2, 16 * a + 4 * j + i + 1) * A.q_scale;
#pragma unroll
      for (int b = 0; b < 2; ++b) acc[a][b][i] *= f;
    }
#pragma unroll
  for (int st = 0; st < kDcTok / 32; ++st) {
    dc_bf16x8 vb[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) vb[b] = dc_ld(vt + (32 * wave + 16 * b + r) * kDcRow + 32 * st + 8 * j);
#pragma unroll
    for (int a = 0; a < 4; ++a) {
      if (16 * a + 15 < 32 * st) continue;                     // all of these keys come after these queries
      const dc_bf16x8 lo = dc_ld(pl + (16 * a + r) * kDcRow + 32 * st + 8 * j), hi = dc_ld(ph + (16 * a + r) * kDcRow + 32 * st + 8 * j);
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo, vb[b], acc[a][b], 0, 0, 0);
        acc[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi, vb[b], acc[a][b], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int a = 0; a < 4; ++a)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int tok = 16 * a + 4 * j + i;
      if (tok >= n) continue;
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const int col = wcol + 16 * b + r;
        if (col < A.dv) A.out[((size_t)(t0 + tok) * A.H + h) * A.dv + col] = acc[a][b][i];
      }
    }
}

}  // namespace xi

using namespace xi;

extern "C" {

// Head sizes the three launches take: whole 16-byte chunks of every row (the caller's strides and pointers too).
int xi_decay_chunks_takes(int dk, int dv) { return dk > 0 && dk <= 256 && dk % 8 == 0 && dv > 0 && dv % 8 == 0; }

// q, k [T, .] with H dk columns and v with H dv, bfloat16 rows `*_stride` elements apart; decay float32 [H]; chunk c is the
// tokens first[c] .. last[c] - 1 (at most 64); portion p is the chunks c0[p] .. c0[p] + count[p] - 1, its request's state at
// state + slots[p] * slot_stride ([H, dk, dv] float32); shares float32 [chunks, H, dk, dv] (scratch); out float32 [T, H, dv].
int xi_decay_chunks(const void* q, long long q_stride, const void* k, long long k_stride, const void* v, long long v_stride,
                    const float* decay, float* state, long long slot_stride, const long long* slots, const int* c0, const int* count,
                    int n_portions, const int* first, const int* last, int n_chunks, float* shares, float* out, int H, int dk, int dv,
                    float q_scale, float k_scale, int act, hipStream_t stream) {
  XI_CHECK(xi_decay_chunks_takes(dk, dv) && H > 0 && H <= 65535, "decay_chunks: heads of %d by %d are not taken", dk, dv);
  XI_CHECK(n_portions >= 0 && n_portions <= 65535 && n_chunks >= n_portions, "decay_chunks: %d chunks of %d portions", n_chunks, n_portions);
  XI_CHECK(q_stride % 8 == 0 && k_stride % 8 == 0 && v_stride % 8 == 0 &&
               ((reinterpret_cast<uintptr_t>(q) | reinterpret_cast<uintptr_t>(k) | reinterpret_cast<uintptr_t>(v)) & 15) == 0,
           "decay_chunks: rows in whole 16-byte chunks");
  XI_CHECK(slot_stride >= (long long)H * dk * dv && decay && state && slots && c0 && count && first && last && shares && out,
           "decay_chunks: an operand is missing");
  XI_CHECK(act == 0 || act == 1, "decay_chunks: unknown activation %d", act);
  if (n_portions == 0) return 0;
  DcArgs A{(const bf16*)q, (const bf16*)k, (const bf16*)v, q_stride, k_stride, v_stride, decay, first, last, shares, shares, out, H, dk, dv,
           act, q_scale, k_scale};
  dim3 grid((unsigned)n_chunks, (unsigned)H, (unsigned)((dv + kDcCols - 1) / kDcCols));
  XI_CHECK(grid.z <= 65535u, "decay_chunks: too many value columns");
#define XI_DC_LAUNCH(KERN, BYTES)                                                                                            \
  do {                                                                                                                       \
    const size_t lds = (BYTES);                                                                                              \
    if (lds > 48 * 1024) {                                                                                                   \
      hipError_t e = hipFuncSetAttribute((const void*)KERN, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);           \
      XI_CHECK(e == hipSuccess, "decay_chunks: cannot get %zu bytes of LDS: %s", lds, hipGetErrorString(e));                 \
    }                                                                                                                        \
    KERN<<<grid, 256, lds, stream>>>(A);                                                                                     \
  } while (0)
#define XI_DC_SHARE(DKT) XI_DC_LAUNCH(decay_share_kernel<DKT>, (size_t)(2 * 16 * DKT + kDcCols) * kDcRow * 2)
#define XI_DC_RESULT(DKS) \
  XI_DC_LAUNCH(decay_result_kernel<DKS>, (size_t)(2 * kDcTok * (32 * DKS + kDcPad) + (kDcCols + 2 * kDcTok) * kDcRow) * 2)
  if (dk <= 32) XI_DC_SHARE(2);
  else if (dk <= 64) XI_DC_SHARE(4);
  else if (dk <= 128) XI_DC_SHARE(8);
  else XI_DC_SHARE(16);
  XI_LAUNCH_CHECK("decay_share");
  const size_t per = (size_t)H * dk * dv;
  decay_carry_kernel<<<dim3((unsigned)((per + 255) / 256), (unsigned)n_portions), 256, 0, stream>>>(state, slot_stride, slots, c0, count,
                                                                                                    first, last, decay, shares, H, dk, dv);
  XI_LAUNCH_CHECK("decay_carry");
  if (dk <= 32) XI_DC_RESULT(1);
  else if (dk <= 64) XI_DC_RESULT(2);
  else if (dk <= 128) XI_DC_RESULT(4);
  else XI_DC_RESULT(8);
  XI_LAUNCH_CHECK("decay_result");
#undef XI_DC_RESULT
#undef XI_DC_SHARE
#undef XI_DC_LAUNCH
  return 0;
}

}  // extern "C"
