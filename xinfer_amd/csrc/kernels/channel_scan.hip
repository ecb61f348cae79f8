// Recurrences of one float32 number a channel, S_t = a_t S_(t-1) + b_t, and what makes their a and b.
//
// Sources of (a_t, b_t):
//   ready    a and b float32 [T, C], made beforehand
//   mingru   from two columns of a packed projection and their biases: a = 1 - sigmoid(z), b = sigmoid(z) c(u) with c(u) =
//            u + 1/2 where u >= 0 and sigmoid(u) where u < 0 (the gates read the current token alone)
// The result is S_t * act(g_t), g columns of a packed projection (with a bias, or none) and act silu or the tanh form of
// gelu, rounded once; the last S of an item goes into its request's slot.
//
// `channel_walk_kernel`: a thread owns V channels of an item (a request's tokens of this step, or one chunk of a long
// portion) and walks its tokens, asking for kScanAhead tokens' operands at once.  Long portions are cut into chunks that
// are walked side by side, in two launches: `channel_share_kernel` leaves every chunk's product of its a and its own sum
// from zero (and a copy of the slot's state, which the last chunk of the second launch overwrites); the walk then starts
// from the shares of the chunks before it, put together in order.  Float32 throughout; the two ways agree to rounding.
//
// The real-gated linear recurrent unit (Griffin): log a = rate * sigmoid(r), a = exp(log a), b = sqrt(1 - a^2) sigmoid(i) u
// with rate = -8 softplus(lambda) a channel, r and i the block-diagonal products of u with their biases.
// `rglru_gates_kernel` makes the two products on the matrix cores and a, b from the float32 sums; `rglru_terms_kernel`
// makes a, b from float32 logits.  1 - a^2 = -expm1(2 log a): no cancellation where a is near 1.
#include "common.h"

namespace xi {

constexpr int kScanAhead = 8;       // tokens whose operands are asked for at once
constexpr int kShareAhead = 16;     // chunks whose shares are

constexpr float kLog2eC = 1.4426950408889634f;

// FAST (the bfloat16 path): the hardware's exponential, reciprocal and square root, each within an ulp of float32; the
// 32-bit path takes the library's.
template <bool FAST> static __device__ __forceinline__ float exp_f(float x) {
  return FAST ? __builtin_amdgcn_exp2f(x * kLog2eC) : expf(x);
}
template <bool FAST> static __device__ __forceinline__ float inv_f(float x) { return FAST ? __builtin_amdgcn_rcpf(x) : 1.f / x; }
template <bool FAST> static __device__ __forceinline__ float sigmoid_f(float x) { return inv_f<FAST>(1.f + exp_f<FAST>(-x)); }

// act 0: none, 1: silu, 2: the tanh form of gelu
template <bool FAST> static __device__ __forceinline__ float gate_of(float g, int act) {
  if (act == 1) return g * sigmoid_f<FAST>(g);
  if (act == 2) {          // 1 + tanh(y) = 2 sigmoid(2 y)
    const float y = 0.7978845608028654f * (g + 0.044715f * g * g * g);
    return FAST ? g * sigmoid_f<FAST>(2.f * y) : 0.5f * g * (1.f + tanhf(y));
  }
  return g;
}

template <int V> static __device__ __forceinline__ void load_run(const float* p, float (&v)[V]) {
  if constexpr (V == 2) {
    const float2 t = *reinterpret_cast<const float2*>(p);
    v[0] = t.x;
    v[1] = t.y;
  } else {
    v[0] = p[0];
  }
}
template <int V> static __device__ __forceinline__ void load_run(const bf16* p, float (&v)[V]) {
  if constexpr (V == 2) {
    const unsigned u = *reinterpret_cast<const unsigned*>(p);
    v[0] = __uint_as_float(u << 16);
    v[1] = __uint_as_float(u & 0xffff0000u);
  } else {
    v[0] = to_float(p[0]);
  }
}
template <int V> static __device__ __forceinline__ void store_run(float* p, const float (&v)[V]) {
  if constexpr (V == 2) *reinterpret_cast<float2*>(p) = make_float2(v[0], v[1]);
  else p[0] = v[0];
}
template <int V> static __device__ __forceinline__ void store_run(bf16* p, const float (&v)[V]) {
  if constexpr (V == 2) {
    const bf16 lo = __float2bfloat16(v[0]), hi = __float2bfloat16(v[1]);
    *reinterpret_cast<unsigned*>(p) = (unsigned)*reinterpret_cast<const unsigned short*>(&lo) |
                                      ((unsigned)*reinterpret_cast<const unsigned short*>(&hi) << 16);
  } else {
    p[0] = __float2bfloat16(v[0]);
  }
}

struct ChannelArgs {
  const float *a, *b;               // ready
  const void *z, *u;                // mingru: the gate's and the candidate's columns
  long long zu_stride;
  const float *z_bias, *u_bias;
  const void* g;
  long long g_stride;
  const float* g_bias;
  int act;
  float* state;
  long long slot_stride;
  const long long* slots;
  const int* cu_q;
  const int* items;                 // int32 [n, 5]: first token, last token, batch row, portion's first item, its items; null: rows of cu_q
  float* share;                     // float32 [n, 2, C]: the chunks' products of a and sums
  float* init;                      // float32 [n, C]: the slots' states, at the portions' first items
  void* out;
  int C;
};

template <typename T, bool MIN, int V>
static __device__ __forceinline__ void operands(const ChannelArgs& A, int t, int c, float (&p)[V], float (&q)[V]) {
  if constexpr (MIN) {
    load_run<V>(static_cast<const T*>(A.z) + (size_t)t * A.zu_stride + c, p);
    load_run<V>(static_cast<const T*>(A.u) + (size_t)t * A.zu_stride + c, q);
  } else {
    load_run<V>(A.a + (size_t)t * A.C + c, p);
    load_run<V>(A.b + (size_t)t * A.C + c, q);
  }
}
template <bool FAST, bool MIN, int V>
static __device__ __forceinline__ void make_terms(float (&p)[V], float (&q)[V], const float (&zb)[V], const float (&ub)[V]) {
  if constexpr (MIN) {
#pragma unroll
    for (int i = 0; i < V; ++i) {
      const float z = p[i] + zb[i], u = q[i] + ub[i];
      const float cand = u >= 0.f ? u + 0.5f : sigmoid_f<FAST>(u);
      const float e = exp_f<FAST>(-fabsf(z)), big = inv_f<FAST>(1.f + e), small = e * big;      // sigmoid(|z|), sigmoid(-|z|)
      p[i] = z >= 0.f ? small : big;          // 1 - sigmoid(z)
      q[i] = (z >= 0.f ? big : small) * cand;
    }
  }
}

struct ChannelItem { int first, last, row, lead, count; };
static __device__ __forceinline__ ChannelItem item_of(const ChannelArgs& A, int n) {
  if (A.items) {
    const int* p = A.items + 5 * (size_t)n;
    return ChannelItem{p[0], p[1], p[2], p[3], p[4]};
  }
  return ChannelItem{A.cu_q[n], A.cu_q[n + 1], n, n, 1};
}

template <typename T, bool MIN, int V>
__global__ __launch_bounds__(256) void channel_share_kernel(const ChannelArgs A) {
  const int n = blockIdx.x;
  const int c = V * (blockIdx.y * 256 + threadIdx.x);
  if (c >= A.C) return;
  const ChannelItem it = item_of(A, n);
  if (it.count <= 1) return;
  if (n == it.lead) {
    float s[V];
    load_run<V>(A.state + (size_t)A.slots[it.row] * A.slot_stride + c, s);
    store_run<V>(A.init + (size_t)n * A.C + c, s);
  }
  if (n + 1 == it.lead + it.count) return;          // a portion's last chunk hands no share on
  float zb[V], ub[V], pa[V], sum[V];
#pragma unroll
  for (int i = 0; i < V; ++i) {
    zb[i] = MIN && A.z_bias ? A.z_bias[c + i] : 0.f;
    ub[i] = MIN && A.u_bias ? A.u_bias[c + i] : 0.f;
    pa[i] = 1.f;
    sum[i] = 0.f;
  }
  for (int t0 = it.first; t0 < it.last; t0 += kScanAhead) {
    float p[kScanAhead][V], q[kScanAhead][V];
#pragma unroll
    for (int k = 0; k < kScanAhead; ++k) operands<T, MIN, V>(A, t0 + k < it.last ? t0 + k : it.last - 1, c, p[k], q[k]);
#pragma unroll
    for (int k = 0; k < kScanAhead; ++k) {
      if (t0 + k >= it.last) break;
      make_terms<sizeof(T) == 2, MIN, V>(p[k], q[k], zb, ub);
#pragma unroll
      for (int i = 0; i < V; ++i) {
        pa[i] *= p[k][i];
        sum[i] = fmaf(p[k][i], sum[i], q[k][i]);
      }
    }
  }
  store_run<V>(A.share + (size_t)n * 2 * A.C + c, pa);
  store_run<V>(A.share + (size_t)n * 2 * A.C + A.C + c, sum);
}

template <typename T, bool MIN, int V>
__global__ __launch_bounds__(256) void channel_walk_kernel(const ChannelArgs A) {
  const int n = blockIdx.x;
  const int c = V * (blockIdx.y * 256 + threadIdx.x);
  if (c >= A.C) return;
  const ChannelItem it = item_of(A, n);
  if (it.last <= it.first) return;
  float* slot = A.state + (size_t)A.slots[it.row] * A.slot_stride + c;
  float zb[V], ub[V], gb[V], s[V];
#pragma unroll
  for (int i = 0; i < V; ++i) {
    zb[i] = MIN && A.z_bias ? A.z_bias[c + i] : 0.f;
    ub[i] = MIN && A.u_bias ? A.u_bias[c + i] : 0.f;
    gb[i] = A.g_bias ? A.g_bias[c + i] : 0.f;
  }
  if (it.count > 1) {
    load_run<V>(A.init + (size_t)it.lead * A.C + c, s);
    for (int j0 = it.lead; j0 < n; j0 += kShareAhead) {           // the chunks before this one, in order
      float pa[kShareAhead][V], sum[kShareAhead][V];
#pragma unroll
      for (int k = 0; k < kShareAhead; ++k) {
        const size_t at = (size_t)(j0 + k < n ? j0 + k : n - 1) * 2 * A.C + c;
        load_run<V>(A.share + at, pa[k]);
        load_run<V>(A.share + at + A.C, sum[k]);
      }
#pragma unroll
      for (int k = 0; k < kShareAhead; ++k) {
        if (j0 + k >= n) break;
#pragma unroll
        for (int i = 0; i < V; ++i) s[i] = fmaf(pa[k][i], s[i], sum[k][i]);
      }
    }
  } else {
    load_run<V>(slot, s);
  }
  const T* g = static_cast<const T*>(A.g);
  T* out = static_cast<T*>(A.out);
  for (int t0 = it.first; t0 < it.last; t0 += kScanAhead) {
    float p[kScanAhead][V], q[kScanAhead][V], gv[kScanAhead][V];
#pragma unroll
    for (int k = 0; k < kScanAhead; ++k) {
      const int t = t0 + k < it.last ? t0 + k : it.last - 1;
      operands<T, MIN, V>(A, t, c, p[k], q[k]);
      load_run<V>(g + (size_t)t * A.g_stride + c, gv[k]);
    }
#pragma unroll
    for (int k = 0; k < kScanAhead; ++k) {
      if (t0 + k >= it.last) break;
      make_terms<sizeof(T) == 2, MIN, V>(p[k], q[k], zb, ub);
      float o[V];
#pragma unroll
      for (int i = 0; i < V; ++i) {
        s[i] = fmaf(p[k][i], s[i], q[k][i]);
        o[i] = s[i] * gate_of<sizeof(T) == 2>(gv[k][i] + gb[i], A.act);
      }
      store_run<V>(out + (size_t)(t0 + k) * A.C + c, o);
    }
  }
  if (n + 1 == it.lead + it.count) store_run<V>(slot, s);
}

// ---- the real-gated linear recurrent unit's a and b ------------------------------------------------------------
template <bool FAST>
static __device__ __forceinline__ void rglru_ab(float r_logit, float i_logit, float rate, float u, float& a, float& b) {
  const float log_a = rate * sigmoid_f<FAST>(r_logit);
  a = exp_f<FAST>(log_a);
  const float x = 2.f * log_a;               // 1 - a^2 = 1 - e^x, x <= 0
  if (FAST) {
    // near 0 by the series of e^x - 1 (x^8 / 8! is below a float32 ulp of it for |x| < 0.35)
    const float series = -x * fmaf(x * 0.5f, fmaf(x * (1.f / 3.f), fmaf(x * 0.25f, fmaf(x * 0.2f, fmaf(x * (1.f / 6.f), fmaf(x, 1.f / 7.f, 1.f), 1.f), 1.f), 1.f), 1.f), 1.f);
    const float rest = x > -0.35f ? series : 1.f - exp_f<true>(x);
    b = __builtin_amdgcn_sqrtf(rest) * sigmoid_f<true>(i_logit) * u;
  } else {
    b = sqrtf(-expm1f(x)) * sigmoid_f<false>(i_logit) * u;
  }
}

// logits float32 [T, blocks, 2, per]: a block's r part, then its i part
template <typename T>
__global__ __launch_bounds__(256) void rglru_terms_kernel(const float* __restrict__ logits, const float* __restrict__ r_bias,
                                                          const float* __restrict__ i_bias, const float* __restrict__ rate,
                                                          const T* __restrict__ u, float* __restrict__ a, float* __restrict__ b,
                                                          int C, int per, long long total) {
  for (long long e = (long long)blockIdx.x * 256 + threadIdx.x; e < total; e += (long long)gridDim.x * 256) {
    const long long t = e / C;
    const int c = (int)(e - t * C);
    const int blk = c / per, k = c - blk * per;
    const float* l = logits + (size_t)t * 2 * C + (size_t)blk * 2 * per + k;
    rglru_ab<false>(l[0] + r_bias[c], l[per] + i_bias[c], rate[c], to_float(u[e]), a[e], b[e]);
  }
}

// A workgroup of four waves: 128 tokens by 32 channels of one block, both products; wave v multiplies tokens 32 v .. 32 v +
// 31 by the 32 rows of each gate's matrix as 4 x 2 v_mfma_f32_16x16x32_bf16 tiles a 32-wide k step (tiles 0, 1: the r
// gate's rows, 2, 3: the i gate's, of the same channels, so that a lane ends with both gates of 4 channels of a token).
// Operands go from memory straight into the lanes, a k step ahead; what lies past K is zeros, rows past the last token or
// channel read the last one again and are dropped.
typedef __attribute__((ext_vector_type(8))) __bf16 cs_bf16x8;
typedef __attribute__((ext_vector_type(4))) float cs_f32x4;

__global__ __launch_bounds__(256) void rglru_gates_kernel(const bf16* __restrict__ u, const bf16* __restrict__ w,
                                                          const float* __restrict__ r_bias, const float* __restrict__ i_bias,
                                                          const float* __restrict__ rate, float* __restrict__ a_out,
                                                          float* __restrict__ b_out, int n_tok, int C, int per) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r = lane & 15, j = lane >> 4;
  const int blk = blockIdx.z, n0 = blockIdx.y * 32, t0 = blockIdx.x * 128 + 32 * wave;
  if (t0 >= n_tok) return;
  const bf16* wb = w + (size_t)blk * 2 * per * per;             // [2, per, per]
  const bf16* xp[2];
  const bf16* wp[4];
#pragma unroll
  for (int tj = 0; tj < 2; ++tj) {
    int t = t0 + 16 * tj + r;
    t = t < n_tok ? t : n_tok - 1;
    xp[tj] = u + (size_t)t * C + (size_t)blk * per + 8 * j;
  }
#pragma unroll
  for (int ti = 0; ti < 4; ++ti) {
    int n = n0 + 16 * (ti & 1) + r;
    n = n < per ? n : per - 1;
    wp[ti] = wb + ((size_t)(ti >> 1) * per + n) * per + 8 * j;
  }
  cs_f32x4 acc[4][2];
#pragma unroll
  for (int ti = 0; ti < 4; ++ti)
#pragma unroll
    for (int tj = 0; tj < 2; ++tj) acc[ti][tj] = cs_f32x4{0.f, 0.f, 0.f, 0.f};
  const cs_bf16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  cs_bf16x8 wa[4], xa[2], wn[4], xn[2];
  const bool on = 8 * j < per;
#pragma unroll
  for (int ti = 0; ti < 4; ++ti) wa[ti] = on ? *reinterpret_cast<const cs_bf16x8*>(wp[ti]) : zero;
#pragma unroll
  for (int tj = 0; tj < 2; ++tj) xa[tj] = on ? *reinterpret_cast<const cs_bf16x8*>(xp[tj]) : zero;
  for (int k0 = 0; k0 < per; k0 += 32) {
    const bool more = k0 + 32 + 8 * j < per;
#pragma unroll
    for (int ti = 0; ti < 4; ++ti) wn[ti] = more ? *reinterpret_cast<const cs_bf16x8*>(wp[ti] + k0 + 32) : zero;
#pragma unroll
    for (int tj = 0; tj < 2; ++tj) xn[tj] = more ? *reinterpret_cast<const cs_bf16x8*>(xp[tj] + k0 + 32) : zero;
#pragma unroll
    for (int ti = 0; ti < 4; ++ti)
#pragma unroll
      for (int tj = 0; tj < 2; ++tj) acc[ti][tj] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wa[ti], xa[tj], acc[ti][tj], 0, 0, 0);
#pragma unroll
    for (int ti = 0; ti < 4; ++ti) wa[ti] = wn[ti];
#pragma unroll
    for (int tj = 0; tj < 2; ++tj) xa[tj] = xn[tj];
  }
  // a lane's 4 values of a tile: token 16 tj + r, channels 16 (ti & 1) + 4 j .. + 3
#pragma unroll
  for (int tj = 0; tj < 2; ++tj) {
    const int t = t0 + 16 * tj + r;
    if (t >= n_tok) continue;
#pragma unroll
    for (int ti = 0; ti < 2; ++ti) {
      const int n = n0 + 16 * ti + 4 * j;
      if (n >= per) continue;                                  // per is a multiple of 8: four channels lie inside or outside together
      const int c = blk * per + n;
      const uint2 uv = *reinterpret_cast<const uint2*>(u + (size_t)t * C + c);
      const float u4[4] = {__uint_as_float(uv.x << 16), __uint_as_float(uv.x & 0xffff0000u), __uint_as_float(uv.y << 16),
                           __uint_as_float(uv.y & 0xffff0000u)};
      float a4[4], b4[4];
#pragma unroll
      for (int i = 0; i < 4; ++i)
        rglru_ab<true>(acc[ti][tj][i] + r_bias[c + i], acc[ti + 2][tj][i] + i_bias[c + i], rate[c + i], u4[i], a4[i], b4[i]);
      *reinterpret_cast<float4*>(a_out + (size_t)t * C + c) = make_float4(a4[0], a4[1], a4[2], a4[3]);
      *reinterpret_cast<float4*>(b_out + (size_t)t * C + c) = make_float4(b4[0], b4[1], b4[2], b4[3]);
    }
  }
}

}  // namespace xi

using namespace xi;

extern "C" {

// a, b float32 [T, C], or (both null) z, u columns of rows of zu_stride elements in `dtype` with biases float32 [C] or
// null; g columns of rows of g_stride elements in `dtype`, g_bias float32 [C] or null, act 0 none, 1 silu, 2 gelu (tanh);
// state float32, slot s at state + s * slot_stride, [C]; slots int64 [B]; cu_q int32 [B + 1]; items int32 [n, 5] or null
// (n = B, a request an item); chunked: some portion has several items, then share float32 [n, 2, C] and init float32
// [n, C] are needed; out [T, C] in `dtype`.
int xi_channel_scan(const float* a, const float* b, const void* z, const void* u, long long zu_stride, const float* z_bias,
                    const float* u_bias, const void* g, long long g_stride, const float* g_bias, int act, float* state,
                    long long slot_stride, const long long* slots, const int* cu_q, const int* items, int n_items, int chunked,
                    float* share, float* init, void* out, int dtype, int C, hipStream_t stream) {
  XI_CHECK(n_items >= 0 && C > 0 && slot_stride >= C && g_stride >= C, "channel_scan: bad sizes items=%d C=%d", n_items, C);
  XI_CHECK((a != nullptr) == (b != nullptr) && (z != nullptr) == (u != nullptr) && (a != nullptr) != (z != nullptr),
           "channel_scan: ready-made terms or a gate's and a candidate's columns");
  XI_CHECK(z == nullptr || zu_stride >= C, "channel_scan: the gate's rows are too short");
  XI_CHECK(g && state && slots && out && (items || cu_q) && act >= 0 && act <= 2, "channel_scan: an operand is missing");
  XI_CHECK(!chunked || (items && share && init), "channel_scan: chunks need their items and places for their shares");
  XI_CHECK(dtype == kF32 || dtype == kBF16, "channel_scan: unknown dtype %d", dtype);
  if (n_items == 0) return 0;
  const uintptr_t run = dtype == kF32 ? 8 : 4;
  auto whole = [](const void* p, uintptr_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; };
  const bool two = C % 2 == 0 && zu_stride % 2 == 0 && g_stride % 2 == 0 && slot_stride % 2 == 0 && whole(a, 8) && whole(b, 8) &&
                   whole(z, run) && whole(u, run) && whole(g, run) && whole(state, 8) && whole(out, run) && whole(share, 8) && whole(init, 8);
  ChannelArgs A{a, b, z, u, zu_stride, z_bias, u_bias, g, g_stride, g_bias, act, state, slot_stride, slots, cu_q, items, share, init, out, C};
  const int per = two ? 512 : 256;
  dim3 grid((unsigned)n_items, (unsigned)((C + per - 1) / per));
  XI_CHECK(grid.y <= 65535u, "channel_scan: too many channels");
#define XI_CS(TT, MIN, V)                                                                   \
  do {                                                                                      \
    if (chunked) channel_share_kernel<TT, MIN, V><<<grid, 256, 0, stream>>>(A);             \
    channel_walk_kernel<TT, MIN, V><<<grid, 256, 0, stream>>>(A);                           \
  } while (0)
#define XI_CS_T(TT)                                    \
  do {                                                 \
    if (a && two) XI_CS(TT, false, 2);                 \
    else if (a) XI_CS(TT, false, 1);                   \
    else if (two) XI_CS(TT, true, 2);                  \
    else XI_CS(TT, true, 1);                           \
  } while (0)
  if (dtype == kF32) XI_CS_T(float);
  else XI_CS_T(bf16);
#undef XI_CS_T
#undef XI_CS
  XI_LAUNCH_CHECK("channel_scan");
  return 0;
}

// logits float32 [T, C / per, 2, per]; r_bias, i_bias, rate float32 [C]; u [T, C] in `dtype`; a, b float32 [T, C].
int xi_rglru_terms(const float* logits, const float* r_bias, const float* i_bias, const float* rate, const void* u, int dtype, float* a,
                   float* b, int n_tok, int C, int per, hipStream_t stream) {
  XI_CHECK(n_tok >= 0 && C > 0 && per > 0 && C % per == 0, "rglru_terms: bad sizes T=%d C=%d block=%d", n_tok, C, per);
  if (n_tok == 0) return 0;
  const long long total = (long long)n_tok * C;
  const long long want = (total + 255) / 256;
  const unsigned grid = (unsigned)(want < 65536 ? want : 65536);
  if (dtype == kF32)
    rglru_terms_kernel<float><<<grid, 256, 0, stream>>>(logits, r_bias, i_bias, rate, (const float*)u, a, b, C, per, total);
  else if (dtype == kBF16)
    rglru_terms_kernel<bf16><<<grid, 256, 0, stream>>>(logits, r_bias, i_bias, rate, (const bf16*)u, a, b, C, per, total);
  else XI_CHECK(false, "rglru_terms: unknown dtype %d", dtype);
  XI_LAUNCH_CHECK("rglru_terms");
  return 0;
}

// bfloat16: u [T, C], w [C / per, 2, per, per] ([out, in], the r gate's matrix first), per a multiple of 8.
int xi_rglru_gates(const void* u, const void* w, const float* r_bias, const float* i_bias, const float* rate, float* a, float* b,
                   int n_tok, int C, int per, hipStream_t stream) {
  XI_CHECK(n_tok >= 0 && C > 0 && per > 0 && per % 8 == 0 && C % per == 0, "rglru_gates: bad sizes T=%d C=%d block=%d", n_tok, C, per);
  XI_CHECK((reinterpret_cast<uintptr_t>(u) & 15) == 0 && (reinterpret_cast<uintptr_t>(w) & 15) == 0, "rglru_gates: rows in whole 16-byte chunks");
  if (n_tok == 0) return 0;
  dim3 grid((unsigned)((n_tok + 127) / 128), (unsigned)((per + 31) / 32), (unsigned)(C / per));
  XI_CHECK(grid.y <= 65535u && grid.z <= 65535u, "rglru_gates: too many channels");
  rglru_gates_kernel<<<grid, 256, 0, stream>>>((const bf16*)u, (const bf16*)w, r_bias, i_bias, rate, a, b, n_tok, C, per);
  XI_LAUNCH_CHECK("rglru_gates");
  return 0;
}

}  // extern "C"
