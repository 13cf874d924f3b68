// Grouped-query attention over a paged pool for layers with sizes of their own: keys and values of different width, an optional
// sliding window (with or without the first tokens of the sequence kept beside it), an optional sink (a score in the softmax denominator
// that carries no value, one for all heads or one a head), an optional soft cap of the scores and an optional sigmoid gate on the output
// (a number an element or a head), all fused into one pass.  Or, instead of the softmax, every key weighted by the sigmoid of its
// score plus an offset a head.
//
//   grouped_kv_store   the keys and values of new tokens into their cache rows
//   grouped_attention  any token mix, split along the keys; matrix form (bf16) and a plain form (every size, bf16 and fp32).  In a
//                      decode batch it reads the step's own keys and values from the projection and stores them on the way
//   grouped_prefill    long extends (bf16): the query heads of one key head are rows of one tile
//
// A cache row is [kv_heads][kd key elements | vd value elements].  kd and vd are multiples of 8; head vectors of other lengths
// come in padded with zeros.  Scores, weights and sums are fp32; a weight enters the bf16 product as a (high, rest) pair.
#include "elem_io.hpp"
#include "mfma_tiles.hpp"
#include "sglang_amd.h"

using namespace sgl_amd;

namespace {

struct GroupedParams {
  const void* q;             // [tokens, heads * kd]
  int64_t q_stride;
  void* cache;               // [slots, kv_heads * (kd + vd)]
  int64_t cache_stride;
  const void *k_new, *v_new; // [tokens, kv_heads * kd], [tokens, kv_heads * vd] of a decode batch, or null: all keys are cached
  int64_t k_stride, v_stride;
  const int64_t* loc;        // [tokens] cache rows of k_new / v_new
  const int32_t* req_to_token;
  int64_t r2t_stride;
  const int64_t* req;        // [segments] row of req_to_token
  const int32_t* tok_seg;    // [tokens] (null: token index)
  const int64_t* positions;  // [tokens]
  const void* gate;          // [tokens, heads * vd], [tokens, heads] (gate_per_head), or null
  int64_t gate_stride;
  void* out;                 // [tokens, heads * vd]
  int64_t o_stride;
  float* part_o;             // [tokens, heads, splits, vd] when splits > 1
  float* part_ml;            // [tokens, heads, splits, 2]
  const int32_t* blocks;     // prefill: [blocks, 2] segment, first token within it
  const int32_t *seg_start, *seg_len;
  int64_t tokens;
  int heads, kv_heads, group, kd, vd, window, splits, block_tokens;
  float scale, sink;         // sink = -inf: none
  const float* sinks;        // [heads], instead of `sink`
  float cap;                 // > 0: scores become cap * tanh(score / cap)
  float softmax_scale, cap_in, cap_out;      // matrix forms: factor in front of 2^x, and of a cap's argument and result
  int gate_per_head;
  int keep;                  // with a window: the first `keep` positions stay visible
  const float* offsets;      // [heads]: weights are sigmoid(score + offset), not normalized; null: softmax
  float out_scale;           // factor on the output
};

__device__ __forceinline__ float sink_of(const GroupedParams& p, int head) { return p.sinks ? p.sinks[head] : p.sink; }

// Products of the matrix form -> what the softmax takes, times `softmax_scale`: log2(e) cap tanh(scale product / cap), with
// tanh x = 1 - 2 / (1 + e^2x): absolute error of a few 2^-24, which is what a score needs.
__device__ __forceinline__ void cap_scores(const GroupedParams& p, f32x4_t& s) {
#pragma unroll
  for (int r = 0; r < 4; ++r) s[r] = p.cap_out - 2.0f * p.cap_out * __builtin_amdgcn_rcpf(1.0f + fast_exp2(s[r] * p.cap_in));
}

// Visible keys are numbered through: the first `kept` positions, then the window's, `gap` further on.
template <bool kKeep = true>
struct KeyMap {
  int kept, gap;
  __device__ __forceinline__ KeyMap(const GroupedParams& p, int window_first) {
    kept = kKeep ? (p.keep < window_first ? p.keep : window_first) : 0;
    gap = window_first - kept;
  }
  __device__ __forceinline__ int operator()(int i) const { return kKeep && i < kept ? i : i + gap; }
};

__device__ __forceinline__ int window_first(const GroupedParams& p, int pos) { return p.window > 0 && pos + 1 > p.window ? pos + 1 - p.window : 0; }

__device__ __forceinline__ void key_range(const GroupedParams& p, const KeyMap<>& key, int pos, int split, int& lo, int& hi) {
  const int n = pos + 1 - key.gap, per = (n + p.splits - 1) / p.splits;
  lo = split * per;
  hi = lo + per < n ? lo + per : n;
}

// 1 / denominator in units of 2^m, for sums taken relative to the maximum m (both in log2): the sink joins here
__device__ __forceinline__ float inverse_sum(float m, float l, float sink) {
  const float s2 = sink * kLog2e;
  const float top = fmaxf(m, s2), f = exp2f(m - top);
  return f / (l * f + exp2f(s2 - top));
}

// what the sums are multiplied with: sigmoid weights are what they are (and come with m = 0)
__device__ __forceinline__ float output_factor(const GroupedParams& p, float m, float l, int head) {
  return p.out_scale * (p.offsets ? 1.0f : inverse_sum(m, l, sink_of(p, head)));
}

template <int VEC, typename T>
__device__ __forceinline__ void store_gated(const GroupedParams& p, int64_t t, int col, float (&v)[VEC]) {
  if (p.gate && p.gate_per_head) {
    const float g = sigmoid_f(ld1(static_cast<const T*>(p.gate) + t * p.gate_stride + col / p.vd));
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] *= g;
  } else if (p.gate) {
    float g[VEC];
    ldv<VEC>(static_cast<const T*>(p.gate) + t * p.gate_stride + col, g);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] *= sigmoid_f(g[j]);
  }
  stv<VEC>(static_cast<T*>(p.out) + t * p.o_stride + col, v);
}

// ---------------------------------------------------------------------------------------------------------------
// 16-byte pieces: ku of a head's key, vu of its value
__global__ __launch_bounds__(256) void grouped_kv_store_kernel(const char* __restrict__ k, int64_t k_bytes, const char* __restrict__ v,
                                                               int64_t v_bytes, char* __restrict__ cache, int64_t cache_bytes,
                                                               const int64_t* __restrict__ loc, int64_t tokens, int kv_heads, int ku, int vu) {
  const int per = kv_heads * (ku + vu);
  const int64_t i = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  const int64_t t = i / per;
  if (t >= tokens) return;
  const int c = static_cast<int>(i - t * per), h = c / (ku + vu), e = c - h * (ku + vu);
  const char* src = e < ku ? k + t * k_bytes + (h * ku + e) * 16 : v + t * v_bytes + (h * vu + (e - ku)) * 16;
  st16(cache + loc[t] * cache_bytes + static_cast<int64_t>(c) * 16, ld16(src));
}

// ---------------------------------------------------------------------------------------------------------------
// Plain form: one workgroup per (token, query head, split); thread = key for the scores, thread = value column for the sums.
template <typename T>
__global__ __launch_bounds__(256) void grouped_attention_plain_kernel(GroupedParams p) {
  extern __shared__ float lds[];
  __shared__ float scratch[16];
  float* q = lds;                 // [kd]
  float* acc = q + p.kd;          // [vd]
  float* sc = acc + p.vd;         // [256]
  const T** kp = reinterpret_cast<const T**>(sc + 256);   // [256] key rows of the tile
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y, split = blockIdx.z, kvh = h / p.group, row_len = p.kd + p.vd;
  const int64_t b = p.tok_seg ? p.tok_seg[t] : t;
  const int32_t* row = p.req_to_token + p.req[b] * p.r2t_stride;
  const T* cache = static_cast<const T*>(p.cache) + static_cast<int64_t>(kvh) * row_len;
  const int64_t pos = p.positions[t];
  const KeyMap<> key(p, window_first(p, static_cast<int>(pos)));
  int lo, hi;
  key_range(p, key, static_cast<int>(pos), split, lo, hi);
  const float offset = p.offsets ? p.offsets[h] : 0.f;
  const T* qp = static_cast<const T*>(p.q) + t * p.q_stride + static_cast<int64_t>(h) * p.kd;
  for (int c = threadIdx.x; c < p.kd; c += 256) q[c] = ld1(qp + c);
  for (int c = threadIdx.x; c < p.vd; c += 256) acc[c] = 0.f;
  __syncthreads();
  float m = p.offsets ? 0.f : -INFINITY, l = 0.f;
  for (int j0 = lo; j0 < hi; j0 += 256) {
    const int j = j0 + threadIdx.x;
    float s = -INFINITY;
    if (j < hi) {
      const T* k = cache + static_cast<int64_t>(row[key(j)]) * p.cache_stride;
      float d = 0.f;
      for (int c = 0; c < p.kd; c += 4) {
        float e[4];
        ld4(k + c, e);
#pragma unroll
        for (int u = 0; u < 4; ++u) d += q[c + u] * e[u];
      }
      s = d * p.scale;
      if (p.cap > 0.f) s = p.cap * tanhf(s / p.cap);
      kp[threadIdx.x] = k;
    }
    float e, fix = 1.0f;
    if (p.offsets) {
      e = j < hi ? sigmoid_f(s + offset) : 0.f;
    } else {
      const float mn = fmaxf(m, block_max(s, scratch));
      e = j < hi ? expf(s - mn) : 0.f;
      fix = expf(m - mn);
      l = l * fix + block_sum(e, scratch);
      m = mn;
    }
    sc[threadIdx.x] = e;
    __syncthreads();
    const int n = hi - j0 < 256 ? hi - j0 : 256;
    for (int c = threadIdx.x; c < p.vd; c += 256) {
      float a = acc[c] * fix;
      for (int i = 0; i < n; ++i) a += sc[i] * ld1(kp[i] + p.kd + c);
      acc[c] = a;
    }
    __syncthreads();
  }
  if (p.splits == 1) {
    const float sink = sink_of(p, h), top = fmaxf(m, sink), f = expf(m - top);
    const float inv = p.out_scale * (p.offsets ? 1.0f : f / (l * f + expf(sink - top)));
    for (int c = threadIdx.x; c < p.vd; c += 256) {
      float v[1] = {acc[c] * inv};
      store_gated<1, T>(p, t, h * p.vd + c, v);
    }
  } else {
    const int64_t part = (t * p.heads + h) * p.splits + split;
    for (int c = threadIdx.x; c < p.vd; c += 256) p.part_o[part * p.vd + c] = acc[c];
    if (threadIdx.x == 0) { p.part_ml[part * 2] = m * kLog2e; p.part_ml[part * 2 + 1] = l; }
  }
}

// Splits of one (token, head), four columns a thread; maxima in log2.  An empty split has m = -inf, l = 0, zero sums.
template <typename T>
__global__ __launch_bounds__(256) void grouped_merge_kernel(GroupedParams p) {
  const int vq = p.vd / 4;
  const int64_t i = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  const int64_t th = i / vq;
  if (th >= p.tokens * p.heads) return;
  const int c = static_cast<int>(i - th * vq) * 4;
  const int64_t t = th / p.heads;
  const int h = static_cast<int>(th - t * p.heads);
  const float* ml = p.part_ml + th * p.splits * 2;
  float m = -INFINITY;
  for (int s = 0; s < p.splits; ++s) m = fmaxf(m, ml[s * 2]);
  float l = 0.f, a[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
  for (int s = 0; s < p.splits; ++s) {
    const float w = exp2f(ml[s * 2] - m);
    float v[4];
    ld4(p.part_o + (th * p.splits + s) * p.vd + c, v);
    l += w * ml[s * 2 + 1];
#pragma unroll
    for (int j = 0; j < 4; ++j) a[j] += w * v[j];
  }
  const float inv = output_factor(p, m, l, h);
#pragma unroll
  for (int j = 0; j < 4; ++j) a[j] *= inv;
  store_gated<4, T>(p, t, h * p.vd + c, a);
}

// ---------------------------------------------------------------------------------------------------------------
// Weights of the scores s[N] (16 keys each, already masked with -inf) of one query a lane against the running maximum m: updates
// m, l, and the sums o by the rescale factor; pf = the weights as product operands, 32 keys each, (high, rest).
template <int N, int VT>
__device__ __forceinline__ void online_softmax(f32x4_t (&s)[N], float sc, float& m, float& l, f32x4_t (&o)[VT], bf16x8_t (&pf)[N / 2][2]) {
  // (the scale is positive: the largest product is the largest score)
  float mx = -INFINITY;
#pragma unroll
  for (int n = 0; n < N; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r) mx = fmaxf(mx, s[n][r]);
  mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
  mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
  const float mn = fmaxf(m, mx * sc);
  const float base = mn == -INFINITY ? 0.f : mn;       // nothing visible yet: all weights zero
  float sum = 0.f;
#pragma unroll
  for (int kk = 0; kk < N / 2; ++kk) {
    uint32_t wh[4], wl[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float e0 = fast_exp2(s[2 * kk + (j >> 1)][2 * (j & 1)] * sc - base);
      const float e1 = fast_exp2(s[2 * kk + (j >> 1)][2 * (j & 1) + 1] * sc - base);
      sum += e0 + e1;
      wh[j] = pack_bf2(e0, e1);
      wl[j] = pack_bf2(e0 - bf_lo(wh[j]), e1 - bf_hi(wh[j]));
    }
    pf[kk][0] = as_frag(U4{wh[0], wh[1], wh[2], wh[3]});
    pf[kk][1] = as_frag(U4{wl[0], wl[1], wl[2], wl[3]});
  }
  if (__any(mn != m)) {                                // some query's maximum moved
    const float fix = fast_exp2(m - base);
    l *= fix;
#pragma unroll
    for (int n = 0; n < VT; ++n) o[n] *= fix;
  }
  l += sum;
  m = mn;
}

// The same with sigmoid weights: `offset` in log2, nothing to normalize.
template <int N>
__device__ __forceinline__ void sigmoid_weights(f32x4_t (&s)[N], float sc, float offset, bf16x8_t (&pf)[N / 2][2]) {
#pragma unroll
  for (int kk = 0; kk < N / 2; ++kk) {
    uint32_t wh[4], wl[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float e0 = __builtin_amdgcn_rcpf(1.0f + fast_exp2(-(s[2 * kk + (j >> 1)][2 * (j & 1)] * sc + offset)));
      const float e1 = __builtin_amdgcn_rcpf(1.0f + fast_exp2(-(s[2 * kk + (j >> 1)][2 * (j & 1) + 1] * sc + offset)));
      wh[j] = pack_bf2(e0, e1);
      wl[j] = pack_bf2(e0 - bf_lo(wh[j]), e1 - bf_hi(wh[j]));
    }
    pf[kk][0] = as_frag(U4{wh[0], wh[1], wh[2], wh[3]});
    pf[kk][1] = as_frag(U4{wl[0], wl[1], wl[2], wl[3]});
  }
}

// Matrix form for few queries a token: a workgroup = one token, 16 query heads of one key head, one split; its four waves take
// 32-key tiles in turn, each with its own running sums (no barrier in the loop), merged at the end.  S^T = K Q^T with the keys
// straight from the cache as operands, O^T = V^T P^T with V^T read transposed from the wave's own LDS tile; a tile's keys and
// values are in flight while the tile before it is multiplied.
template <int KS, int VT, bool kSigmoid>
__global__ __launch_bounds__(256, 2) void grouped_attention_mfma_kernel(GroupedParams p) {
  constexpr int VLS = VT * 16 + 8, kRegion = VT * 512 + 256, VP = VT / 4;      // (a region also holds [16][VT * 16] fp32 sums)
  __shared__ __attribute__((aligned(16))) uint16_t smem[4 * kRegion];
  __shared__ float wm[4][16], wl[4][16];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), i16 = lane & 15, g = lane >> 4;
  const int64_t t = blockIdx.x;
  const int row_blocks = (p.group + 15) / 16;
  const int kvh = blockIdx.y / row_blocks, h0 = (blockIdx.y % row_blocks) * 16, split = blockIdx.z;
  const int head_n = p.group - h0 < 16 ? p.group - h0 : 16;                    // heads of this workgroup
  const int64_t b = p.tok_seg ? p.tok_seg[t] : t;
  const int32_t* row = p.req_to_token + p.req[b] * p.r2t_stride;
  const int64_t head_off = static_cast<int64_t>(kvh) * (p.kd + p.vd);
  const uint16_t* cache = static_cast<const uint16_t*>(p.cache) + head_off;
  const int pos = static_cast<int>(p.positions[t]);
  const KeyMap<> key(p, window_first(p, pos));
  const int newest = pos - key.gap;                    // number of the token itself
  int lo, hi;
  key_range(p, key, pos, split, lo, hi);
  const uint16_t *kn = nullptr, *vn = nullptr;
  if (p.k_new) {
    kn = static_cast<const uint16_t*>(p.k_new) + t * p.k_stride + static_cast<int64_t>(kvh) * p.kd;
    vn = static_cast<const uint16_t*>(p.v_new) + t * p.v_stride + static_cast<int64_t>(kvh) * p.vd;
    if (h0 == 0 && split == 0) {                       // (nobody reads this row in this launch)
      uint16_t* dst = static_cast<uint16_t*>(p.cache) + p.loc[t] * p.cache_stride + head_off;
      for (int i = threadIdx.x * 8; i < p.kd + p.vd; i += 2048) st16(dst + i, ld16(i < p.kd ? kn + i : vn + (i - p.kd)));
    }
  }
  bf16x8_t q[KS];
  {
    const uint16_t* qr = static_cast<const uint16_t*>(p.q) + t * p.q_stride +
                         static_cast<int64_t>(kvh * p.group + h0 + (i16 < head_n ? i16 : head_n - 1)) * p.kd;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int e = 32 * k + 8 * g;
      q[k] = as_frag(keep_if(ld16(e < p.kd ? qr + e : qr), e < p.kd));
    }
  }
  uint16_t* vt = smem + wave * kRegion;
  f32x4_t o[VT];
#pragma unroll
  for (int n = 0; n < VT; ++n) o[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = kSigmoid ? 0.f : -INFINITY, l = 0.f;
  const float offset = kSigmoid ? p.offsets[kvh * p.group + h0 + (i16 < head_n ? i16 : head_n - 1)] * kLog2e : 0.f;
  const int first = lo + 32 * wave;
  int slot[2];
  U4 kreg[2][KS], vreg[4][VP];
  auto slots = [&](int j0) __attribute__((always_inline)) {                    // keys j0 + 16 n + i16, clamped to the last one
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int j = j0 + 16 * n + i16;
      slot[n] = row[key(j < hi ? j : hi - 1)];
    }
  };
  auto load = [&](int j0) __attribute__((always_inline)) {
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      int j = j0 + 16 * n + i16;
      j = j < hi ? j : hi - 1;
      const uint16_t* kr = kn && j == newest ? kn : cache + static_cast<int64_t>(slot[n]) * p.cache_stride;
#pragma unroll
      for (int k = 0; k < KS; ++k) kreg[n][k] = ld16(32 * k + 8 * g < p.kd ? kr + 32 * k + 8 * g : kr);
    }
#pragma unroll
    for (int w = 0; w < 4; ++w) {                                              // value rows 8 w + lane / 8, eight lanes a row
      int j = j0 + 8 * w + (lane >> 3);
      j = j < hi ? j : hi - 1;
      const int sl = __shfl(slot[w >> 1], (w & 1) * 8 + (lane >> 3), 64);
      const uint16_t* vr = vn && j == newest ? vn : cache + static_cast<int64_t>(sl) * p.cache_stride + p.kd;
#pragma unroll
      for (int i = 0; i < VP; ++i) {
        const int e = (lane & 7) * 8 + 64 * i;
        vreg[w][i] = ld16(e < p.vd ? vr + e : vr);
      }
    }
  };
  if (first < hi) {
    slots(first);
    load(first);
    slots(first + 128);
  }
  for (int j0 = first; j0 < hi; j0 += 128) {
#pragma unroll
    for (int w = 0; w < 4; ++w)
#pragma unroll
      for (int i = 0; i < VP; ++i) st16(vt + (8 * w + (lane >> 3)) * VLS + (lane & 7) * 8 + 64 * i, vreg[w][i]);
    f32x4_t s[2];
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      s[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k) s[n] = mfma_bf16(as_frag(kreg[n][k]), q[k], s[n]);
    }
    if (j0 + 128 < hi) {
      load(j0 + 128);
      slots(j0 + 256);
    }
    if (p.cap > 0.f) {
#pragma unroll
      for (int n = 0; n < 2; ++n) cap_scores(p, s[n]);
    }
    if (j0 + 32 > hi) {
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (j0 + 16 * n + 4 * g + r >= hi) s[n][r] = -INFINITY;
    }
    bf16x8_t pf[1][2];
    if constexpr (kSigmoid) sigmoid_weights<2>(s, p.softmax_scale, offset, pf);
    else online_softmax<2, VT>(s, p.softmax_scale, m, l, o, pf);
    asm volatile("" ::: "memory");                     // (the tile is this wave's own; LDS serves a wave in order)
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int n = 0; n < VT; ++n) {
      const bf16x8_t v = read_transposed(vt, VLS, 0, 16 * n, i16, g);
      o[n] = mfma_bf16(v, pf[0][0], o[n]);
      o[n] = mfma_bf16(v, pf[0][1], o[n]);
    }
    asm volatile("" ::: "memory");
    __builtin_amdgcn_wave_barrier();
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (g == 0) { wm[wave][i16] = m; wl[wave][i16] = l; }
  __syncthreads();
  float top = fmaxf(fmaxf(wm[0][i16], wm[1][i16]), fmaxf(wm[2][i16], wm[3][i16]));
  top = top == -INFINITY ? 0.f : top;                  // an empty split
  const float mine = fast_exp2(m - top);
  float* acc = reinterpret_cast<float*>(vt);           // [16 heads][VT * 16], relative to the common maximum
#pragma unroll
  for (int n = 0; n < VT; ++n) {
    const float v[4] = {o[n][0] * mine, o[n][1] * mine, o[n][2] * mine, o[n][3] * mine};
    st4(acc + i16 * (VT * 16) + 16 * n + 4 * g, v);
  }
  __syncthreads();
  constexpr int CQ = VT * 4;                           // groups of four columns a head
  for (int i = threadIdx.x; i < head_n * CQ; i += 256) {
    const int hd = i / CQ, c = (i % CQ) * 4;
    if (c >= p.vd) continue;
    float mt = -INFINITY;
#pragma unroll
    for (int w = 0; w < 4; ++w) mt = fmaxf(mt, wm[w][hd]);
    float lt = 0.f, a[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      lt += wl[w][hd] * fast_exp2(wm[w][hd] - (mt == -INFINITY ? 0.f : mt));
      float v[4];
      ld4(reinterpret_cast<const float*>(smem + w * kRegion) + hd * (VT * 16) + c, v);
#pragma unroll
      for (int j = 0; j < 4; ++j) a[j] += v[j];
    }
    const int head = kvh * p.group + h0 + hd;
    if (p.splits == 1) {
      const float inv = output_factor(p, mt, lt, head);
#pragma unroll
      for (int j = 0; j < 4; ++j) a[j] *= inv;
      store_gated<4, uint16_t>(p, t, head * p.vd + c, a);
    } else {
      const int64_t part = (t * p.heads + head) * p.splits + split;
      st4(p.part_o + part * p.vd + c, a);
      if (c == 0) { p.part_ml[part * 2] = mt; p.part_ml[part * 2 + 1] = lt; }
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// Long extends: a workgroup = 128 rows of one key head, row = (token, query head of the group), a wave = 32 rows; key tiles of 64
// double-buffered in LDS, the next tile's rows in registers meanwhile; two workgroups a compute unit, so that one multiplies
// while the other forms weights.  S^T = K Q^T leaves the weights of a row in the lane that
// needs them for O^T = V^T P^T, so they never touch LDS.
constexpr int kPfThreads = 256, kPfRows = 128, kPfTile = 64, kPfPass = kPfThreads / 8;

template <int KS, int VT, bool kSigmoid, bool kKeep>
__global__ __launch_bounds__(kPfThreads, 2) void grouped_prefill_kernel(GroupedParams p) {
  constexpr int KLS = KS * 32 + 8, VLS = VT * 16 + 8, KP = KS / 2, VP = VT / 4, NP = kPfTile / kPfPass;
  __shared__ __attribute__((aligned(16))) uint16_t kimg[2][kPfTile * KLS];
  __shared__ __attribute__((aligned(16))) uint16_t vimg[2][kPfTile * VLS];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), i16 = lane & 15, g = lane >> 4;
  const int kvh = blockIdx.x;
  const int b = p.blocks[2 * blockIdx.y], q0 = p.blocks[2 * blockIdx.y + 1];
  const int64_t t0 = p.seg_start[b] + q0;
  const int left = p.seg_len[b] - q0;
  const int last = (left < p.block_tokens ? left : p.block_tokens) - 1;        // last token of the block, from its first
  const int pos0 = static_cast<int>(p.positions[t0]);
  const KeyMap<kKeep> key(p, window_first(p, pos0));
  const int end = pos0 + last + 1 - key.gap;           // keys the block sees
  const int32_t* row = p.req_to_token + p.req[b] * p.r2t_stride;
  const uint16_t* cache = static_cast<const uint16_t*>(p.cache) + static_cast<int64_t>(kvh) * (p.kd + p.vd);

  bf16x8_t q[2][KS];
  int qtok[2], qhead[2];
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int r = 32 * wave + 16 * c + i16;
    qtok[c] = r / p.group;
    qhead[c] = r - qtok[c] * p.group;
    const int tk = qtok[c] <= last ? qtok[c] : last;                           // (rows behind the block are computed and never stored)
    const uint16_t* qr = static_cast<const uint16_t*>(p.q) + (t0 + tk) * p.q_stride + static_cast<int64_t>(kvh * p.group + qhead[c]) * p.kd;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int e = 32 * k + 8 * g;
      q[c][k] = as_frag(keep_if(ld16(e < p.kd ? qr + e : qr), e < p.kd));
    }
  }
  const int tok_first = 32 * wave / p.group, tok_last = (32 * wave + 31) / p.group;
  const bool wave_live = tok_first <= last;
  const int wave_first = pos0 + tok_first, wave_last = pos0 + (tok_last < last ? tok_last : last);
  const int r_row = threadIdx.x >> 3, r_col = (threadIdx.x & 7) * 8;           // eight threads a key row
  U4 kreg[NP][KP], vreg[NP][VP];
  int slot[NP];
  auto next_slot = [&](int j0) __attribute__((always_inline)) {
#pragma unroll
    for (int w = 0; w < NP; ++w) {
      const int j = j0 + w * kPfPass + r_row;
      slot[w] = row[key(j < end ? j : end - 1)];
    }
  };
  // (addresses are clamped, never predicated: all loads stay in flight; columns behind kd meet zeros of the query, columns behind
  // vd are not stored, keys behind the last are masked)
  auto load = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int w = 0; w < NP; ++w) {
      const uint16_t* kr = cache + static_cast<int64_t>(slot[w]) * p.cache_stride;
#pragma unroll
      for (int i = 0; i < KP; ++i) kreg[w][i] = ld16(r_col + 64 * i < p.kd ? kr + r_col + 64 * i : kr);
#pragma unroll
      for (int i = 0; i < VP; ++i) vreg[w][i] = ld16(kr + p.kd + (r_col + 64 * i < p.vd ? r_col + 64 * i : 0));
    }
  };
  f32x4_t o[2][VT];
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
  float offset[2] = {0.f, 0.f};
  if constexpr (kSigmoid) {
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      m[c] = 0.f;
      offset[c] = p.offsets[kvh * p.group + qhead[c]] * kLog2e;
    }
  }
#pragma unroll
  for (int c = 0; c < 2; ++c)
#pragma unroll
    for (int n = 0; n < VT; ++n) o[c][n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  next_slot(0);
  load();
  next_slot(kPfTile);
  int image = 0;
  for (int j0 = 0; j0 < end; j0 += kPfTile, image ^= 1) {
    // (the barrier of the tile before this one lies behind every read of this image)
    uint16_t *kt = kimg[image], *vt = vimg[image];
#pragma unroll
    for (int w = 0; w < NP; ++w) {
#pragma unroll
      for (int i = 0; i < KP; ++i) st16(kt + (w * kPfPass + r_row) * KLS + r_col + 64 * i, kreg[w][i]);
#pragma unroll
      for (int i = 0; i < VP; ++i) st16(vt + (w * kPfPass + r_row) * VLS + r_col + 64 * i, vreg[w][i]);
    }
    __syncthreads();
    if (j0 + kPfTile < end) {
      load();
      next_slot(j0 + 2 * kPfTile);
    }
    // a wave leaves out tiles none of its rows sees
    const int key0 = key(j0), key1 = key(j0 + kPfTile - 1);
    if (!wave_live || key0 > wave_last || (p.window > 0 && key1 <= wave_first - p.window && (!kKeep || key0 >= p.keep))) continue;
    f32x4_t s[2][4];
#pragma unroll
    for (int n = 0; n < 4; ++n) {
      s[0][n] = s[1][n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const bf16x8_t a = as_frag(ld16(kt + (16 * n + i16) * KLS + 32 * k + 8 * g));
        s[0][n] = mfma_bf16(a, q[0][k], s[0][n]);
        s[1][n] = mfma_bf16(a, q[1][k], s[1][n]);
      }
    }
    if (p.cap > 0.f) {
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        cap_scores(p, s[0][n]);
        cap_scores(p, s[1][n]);
      }
    }
    if (key1 > wave_first || (p.window > 0 && key0 <= wave_last - p.window)) {
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        const int qpos = pos0 + qtok[c];
#pragma unroll
        for (int n = 0; n < 4; ++n)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = key(j0 + 16 * n + 4 * g + r);
            if (j > qpos || (p.window > 0 && j <= qpos - p.window && (!kKeep || j >= p.keep))) s[c][n][r] = -INFINITY;
          }
      }
    }
    bf16x8_t pf[2][2][2];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      if constexpr (kSigmoid) sigmoid_weights<4>(s[c], p.softmax_scale, offset[c], pf[c]);
      else online_softmax<4, VT>(s[c], p.softmax_scale, m[c], l[c], o[c], pf[c]);
    }
#pragma unroll
    for (int n = 0; n < VT; ++n)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const bf16x8_t v = read_transposed(vt, VLS, 32 * kk, 16 * n, i16, g);
#pragma unroll
        for (int c = 0; c < 2; ++c) {
          o[c][n] = mfma_bf16(v, pf[c][kk][0], o[c][n]);
          o[c][n] = mfma_bf16(v, pf[c][kk][1], o[c][n]);
        }
      }
  }
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    float sum = l[c];
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (qtok[c] > last) continue;
    const float inv = output_factor(p, m[c], sum, kvh * p.group + qhead[c]);
#pragma unroll
    for (int n = 0; n < VT; ++n) {
      const int e = 16 * n + 4 * g;
      if (e < p.vd) {
        float v[4] = {o[c][n][0] * inv, o[c][n][1] * inv, o[c][n][2] * inv, o[c][n][3] * inv};
        store_gated<4, uint16_t>(p, t0 + qtok[c], (kvh * p.group + qhead[c]) * p.vd + e, v);
      }
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
template <int KS, bool kSigmoid>
void launch_mfma(const GroupedParams& p, const dim3& grid, hipStream_t st) {
  if (p.vd <= 64) hipLaunchKernelGGL((grouped_attention_mfma_kernel<KS, 4, kSigmoid>), grid, dim3(256), 0, st, p);
  else if (p.vd <= 128) hipLaunchKernelGGL((grouped_attention_mfma_kernel<KS, 8, kSigmoid>), grid, dim3(256), 0, st, p);
  else hipLaunchKernelGGL((grouped_attention_mfma_kernel<KS, 16, kSigmoid>), grid, dim3(256), 0, st, p);
}

template <bool kSigmoid>
void launch_mfma(const GroupedParams& p, const dim3& grid, hipStream_t st) {
  if (p.kd <= 64) launch_mfma<2, kSigmoid>(p, grid, st);
  else if (p.kd <= 128) launch_mfma<4, kSigmoid>(p, grid, st);
  else launch_mfma<8, kSigmoid>(p, grid, st);
}

template <int KS, bool kSigmoid, bool kKeep>
void launch_prefill(const GroupedParams& p, const dim3& grid, hipStream_t st) {
  if (p.vd <= 64) hipLaunchKernelGGL((grouped_prefill_kernel<KS, 4, kSigmoid, kKeep>), grid, dim3(kPfThreads), 0, st, p);
  else hipLaunchKernelGGL((grouped_prefill_kernel<KS, 8, kSigmoid, kKeep>), grid, dim3(kPfThreads), 0, st, p);
}

// (sigmoid weights: one form, with or without kept keys)
template <bool kSigmoid, bool kKeep>
void launch_prefill(const GroupedParams& p, const dim3& grid, hipStream_t st) {
  if (p.kd <= 64) launch_prefill<2, kSigmoid, kKeep>(p, grid, st);
  else if (p.kd <= 128) launch_prefill<4, kSigmoid, kKeep>(p, grid, st);
  else launch_prefill<8, kSigmoid, kKeep>(p, grid, st);
}

// keys the window keeps, weights that are sigmoids, factor on the output
bool set_variants(GroupedParams& p, int keep, const float* offsets, float out_scale) {
  p.keep = p.window > 0 ? keep : 0; p.offsets = offsets; p.out_scale = out_scale;
  return keep >= 0 && !(offsets && (p.cap > 0.f || p.sinks || p.sink > -INFINITY));
}

void set_scores(GroupedParams& p, float scale, float cap) {
  p.scale = scale; p.cap = cap;
  p.softmax_scale = cap > 0.f ? 1.0f : scale * kLog2e;
  p.cap_in = cap > 0.f ? 2.0f * kLog2e * scale / cap : 0.f;
  p.cap_out = kLog2e * cap;
}

bool whole_vectors(const GroupedParams& p) {
  return p.kd % 8 == 0 && p.vd % 8 == 0 && p.q_stride % 8 == 0 && p.cache_stride % 8 == 0 && p.o_stride % 4 == 0 && (p.gate_per_head || (p.gate_stride % 4 == 0 && aligned_to(p.gate, 8))) &&
         p.k_stride % 8 == 0 && p.v_stride % 8 == 0 && aligned_to(p.q, 16) && aligned_to(p.cache, 16) && aligned_to(p.k_new, 16) &&
         aligned_to(p.v_new, 16) && aligned_to(p.out, 8) && aligned_to(p.part_o, 16);
}

}  // namespace

extern "C" {

int sgl_amd_grouped_kv_store(int is_f32, const void* k, int64_t k_stride, const void* v, int64_t v_stride, void* cache, int64_t cache_stride,
                             const int64_t* loc, int64_t tokens, int kv_heads, int kd, int vd, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  const int64_t es = is_f32 ? 4 : 2;
  SGL_CHECK_ARG(k && v && cache && loc && kv_heads > 0 && kd > 0 && vd > 0 && kd % 8 == 0 && vd % 8 == 0 && cache_stride >= kv_heads * (kd + vd),
                "grouped_kv_store: %d heads of %d + %d in rows of %lld", kv_heads, kd, vd, (long long)cache_stride);
  SGL_CHECK_ARG(k_stride * es % 16 == 0 && v_stride * es % 16 == 0 && cache_stride * es % 16 == 0 && aligned_to(k, 16) && aligned_to(v, 16) &&
                    aligned_to(cache, 16), "grouped_kv_store: rows of whole 16-byte vectors");
  if (tokens <= 0) return 0;
  const int ku = kd * static_cast<int>(es) / 16, vu = vd * static_cast<int>(es) / 16;
  const int64_t n = tokens * kv_heads * (ku + vu);
  hipLaunchKernelGGL(grouped_kv_store_kernel, dim3(static_cast<unsigned>((n + 255) / 256)), dim3(256), 0, as_stream(stream),
                     static_cast<const char*>(k), k_stride * es, static_cast<const char*>(v), v_stride * es, static_cast<char*>(cache),
                     cache_stride * es, loc, tokens, kv_heads, ku, vu);
  SGL_CHECK_LAUNCH("grouped_kv_store");
  return 0;
}

int sgl_amd_grouped_attention_matrix_form(int kd, int vd) { return kd % 8 == 0 && vd % 8 == 0 && kd <= 256 && vd <= 256 ? 1 : 0; }
int sgl_amd_grouped_prefill_supported(int kd, int vd, int group) {
  return kd % 8 == 0 && vd % 8 == 0 && kd <= 256 && vd <= 128 && group >= 1 && group <= kPfRows ? 1 : 0;
}
int sgl_amd_grouped_prefill_rows(void) { return kPfRows; }

int sgl_amd_grouped_attention(int is_f32, const void* q, int64_t q_stride, void* cache, int64_t cache_stride, const void* k_new, int64_t k_stride,
                              const void* v_new, int64_t v_stride, const int64_t* loc, const int32_t* req_to_token, int64_t r2t_stride,
                              const int64_t* req_pool_indices, const int32_t* tok_seg, const int64_t* positions, const void* gate,
                              int64_t gate_stride, void* out, int64_t o_stride, float* part_o, float* part_ml, int64_t tokens, int heads,
                              int kv_heads, int kd, int vd, int window, int splits, float scale, float sink, const float* sinks, float cap,
                              int gate_per_head, int plain, int keep, const float* offsets, float out_scale, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(q && cache && req_to_token && req_pool_indices && positions && out, "grouped_attention: null operand");
  SGL_CHECK_ARG(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && heads <= 65535 && kd > 0 && vd > 0 && kd % 4 == 0 && vd % 4 == 0 &&
                    cache_stride >= kv_heads * (kd + vd) && splits >= 1 && splits <= 64,
                "grouped_attention: %d / %d heads of %d + %d, %d splits", heads, kv_heads, kd, vd, splits);
  SGL_CHECK_ARG(splits == 1 || (part_o && part_ml), "grouped_attention: split launches need their workspaces");
  if (tokens <= 0) return 0;
  GroupedParams p{};
  p.q = q; p.q_stride = q_stride; p.cache = cache; p.cache_stride = cache_stride; p.k_new = k_new; p.v_new = v_new; p.k_stride = k_stride;
  p.v_stride = v_stride; p.loc = loc; p.req_to_token = req_to_token; p.r2t_stride = r2t_stride; p.req = req_pool_indices; p.tok_seg = tok_seg;
  p.positions = positions; p.gate = gate; p.gate_stride = gate_stride; p.out = out; p.o_stride = o_stride; p.part_o = part_o; p.part_ml = part_ml;
  p.tokens = tokens; p.heads = heads; p.kv_heads = kv_heads; p.group = heads / kv_heads; p.kd = kd; p.vd = vd; p.window = window;
  p.splits = splits; p.sink = sink; p.sinks = sinks; p.gate_per_head = gate_per_head;
  set_scores(p, scale, cap);
  SGL_CHECK_ARG(set_variants(p, keep, offsets, out_scale), "grouped_attention: %d kept keys; sigmoid weights take no cap and no sink", keep);
  hipStream_t st = as_stream(stream);
  const bool matrix = !is_f32 && !plain && sgl_amd_grouped_attention_matrix_form(kd, vd) && whole_vectors(p) && scale > 0.f;
  SGL_CHECK_ARG(!k_new || (matrix && v_new && loc && !tok_seg), "grouped_attention: only the matrix form of a decode batch takes keys and values that are not stored yet");
  if (matrix) {
    const dim3 grid(static_cast<unsigned>(tokens), kv_heads * ((p.group + 15) / 16), splits);
    if (offsets) launch_mfma<true>(p, grid, st);
    else launch_mfma<false>(p, grid, st);
  } else {
    const dim3 grid(static_cast<unsigned>(tokens), heads, splits);
    const size_t lds = (static_cast<size_t>(kd) + vd + 256) * 4 + 256 * 8;
    SGL_CHECK_ARG(lds <= 64 * 1024 - 256, "grouped_attention: head sizes %d + %d need %zu bytes of LDS", kd, vd, lds);
    const size_t al = is_f32 ? 16 : 8;
    SGL_CHECK_ARG(cache_stride % 4 == 0 && aligned_to(cache, al) && o_stride % 4 == 0 && aligned_to(out, al) &&
                      (gate_per_head || (gate_stride % 4 == 0 && aligned_to(gate, al))),
                  "grouped_attention: rows of whole 4-element pieces");
    if (is_f32) hipLaunchKernelGGL((grouped_attention_plain_kernel<float>), grid, dim3(256), lds, st, p);
    else hipLaunchKernelGGL((grouped_attention_plain_kernel<uint16_t>), grid, dim3(256), lds, st, p);
  }
  SGL_CHECK_LAUNCH("grouped_attention");
  if (splits > 1) {
    const dim3 grid(static_cast<unsigned>((tokens * heads * (vd / 4) + 255) / 256));
    if (is_f32) hipLaunchKernelGGL((grouped_merge_kernel<float>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((grouped_merge_kernel<uint16_t>), grid, dim3(256), 0, st, p);
    SGL_CHECK_LAUNCH("grouped_attention (merge)");
  }
  return 0;
}

int sgl_amd_grouped_prefill(const void* q, int64_t q_stride, const void* cache, int64_t cache_stride, const int32_t* req_to_token,
                            int64_t r2t_stride, const int64_t* req_pool_indices, const int32_t* blocks, int num_blocks,
                            const int32_t* seg_start, const int32_t* seg_len, const int64_t* positions, const void* gate, int64_t gate_stride,
                            void* out, int64_t o_stride, int heads, int kv_heads, int kd, int vd, int window, float scale, float sink,
                            const float* sinks, float cap, int gate_per_head, int keep, const float* offsets, float out_scale, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(q && cache && req_to_token && req_pool_indices && blocks && seg_start && seg_len && positions && out, "grouped_prefill: null operand");
  SGL_CHECK_ARG(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && sgl_amd_grouped_prefill_supported(kd, vd, heads / kv_heads) &&
                    cache_stride >= kv_heads * (kd + vd) && num_blocks <= 65535 && scale > 0.f,
                "grouped_prefill: %d / %d heads of %d + %d, %d blocks, scale %g", heads, kv_heads, kd, vd, num_blocks, scale);
  if (num_blocks <= 0) return 0;
  GroupedParams p{};
  p.q = q; p.q_stride = q_stride; p.cache = const_cast<void*>(cache); p.cache_stride = cache_stride; p.req_to_token = req_to_token;
  p.r2t_stride = r2t_stride; p.req = req_pool_indices; p.positions = positions; p.gate = gate; p.gate_stride = gate_stride; p.out = out;
  p.o_stride = o_stride; p.blocks = blocks; p.seg_start = seg_start; p.seg_len = seg_len; p.heads = heads; p.kv_heads = kv_heads;
  p.group = heads / kv_heads; p.kd = kd; p.vd = vd; p.window = window; p.splits = 1; p.block_tokens = kPfRows / p.group; p.sink = sink;
  p.sinks = sinks; p.gate_per_head = gate_per_head;
  set_scores(p, scale, cap);
  SGL_CHECK_ARG(set_variants(p, keep, offsets, out_scale), "grouped_prefill: %d kept keys; sigmoid weights take no cap and no sink", keep);
  SGL_CHECK_ARG(whole_vectors(p), "grouped_prefill: rows of whole 16-byte vectors");
  const dim3 grid(kv_heads, num_blocks);
  hipStream_t st = as_stream(stream);
  if (offsets) launch_prefill<true, true>(p, grid, st);
  else if (p.keep > 0) launch_prefill<false, true>(p, grid, st);
  else launch_prefill<false, false>(p, grid, st);
  SGL_CHECK_LAUNCH("grouped_prefill");
  return 0;
}

}  // extern "C"
