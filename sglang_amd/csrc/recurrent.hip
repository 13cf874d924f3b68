// Recurrent mixers over a ragged batch: the short causal convolution in front of them, and the Mamba-2, gated-delta-rule and
// matrix-memory state updates in their token-by-token form (decode steps and short portions; prefill-sized portions:
// recurrent_chunk.hip).  And the token shift of ragged batches, whose state is one row a request.
//
// A batch is a list of segments (one per request): tokens [seg_start[b], seg_start[b] + seg_len[b]) of the packed rows; both
// pointers null = one token per request.  Request b's state lives in slot slots[b].  A segment that begins at position 0
// starts from zero whatever the slot holds, so a slot is never cleared.
//
// Convolution history is a ring of `taps` rows per slot, position p in row p % taps: the row a token writes is never one the
// same token reads, so a decode step convolves and stores in one launch without ordering its threads.
#include "elem_io.hpp"
#include "sglang_amd.h"

using namespace sgl_amd;

namespace {

struct ConvParams {
  const void* x;             // [tokens, channels]
  int64_t x_stride;
  const float* w;            // [taps, channels]: row 0 = the current token
  const float* bias;         // optional [channels]
  void* state;               // [slots, taps, channels]
  const int64_t* slots;      // [segments]
  const int64_t* positions;  // [tokens]
  const int32_t* tok_seg;    // [tokens] segment of a token (null: token index)
  const int32_t* seg_start;  // [segments] (null: token index)
  void* out;
  int64_t out_stride;
  int64_t tokens;
  int channels, taps, store;
};

// A thread owns VEC channels of TOK consecutive tokens.  TAPS > 0: the history length is a compile-time constant, and when the
// tokens and their history are consecutive rows of one segment every input is read once, all reads in flight together; at a
// segment's start (and for TAPS = 0, any length) inputs are found one by one, in the packed rows or in the ring.
template <typename T, int VEC, int TAPS, int TOK>
__global__ __launch_bounds__(256) void conv_silu_kernel(ConvParams p) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (c >= p.channels) return;
  const T* x = static_cast<const T*>(p.x) + c;
  T* out = static_cast<T*>(p.out) + c;
  T* state = static_cast<T*>(p.state) + c;
  const int64_t t0 = static_cast<int64_t>(blockIdx.y) * TOK;
  const int taps = TAPS > 0 ? TAPS : p.taps;
  float bias[VEC];
#pragma unroll
  for (int j = 0; j < VEC; ++j) bias[j] = 0.f;
  if (p.bias) ldv<VEC>(p.bias + c, bias);
  if constexpr (TAPS > 0 && TOK > 1) {
    const int64_t b0 = p.tok_seg[t0];
    if (t0 + TOK <= p.tokens && p.tok_seg[t0 + TOK - 1] == b0 && t0 - p.seg_start[b0] >= TAPS - 1) {
      float w[TAPS][VEC], v[TOK + TAPS - 1][VEC];
#pragma unroll
      for (int i = 0; i < TOK + TAPS - 1; ++i) ldv<VEC>(x + (t0 + i - (TAPS - 1)) * p.x_stride, v[i]);
#pragma unroll
      for (int d = 0; d < TAPS; ++d) ldv<VEC>(p.w + static_cast<int64_t>(d) * p.channels + c, w[d]);
#pragma unroll
      for (int i = 0; i < TOK; ++i) {
        float o[VEC];
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          float acc = bias[j];
#pragma unroll
          for (int d = 0; d < TAPS; ++d) acc += w[d][j] * v[i + TAPS - 1 - d][j];
          o[j] = silu_f(acc);
        }
        stv<VEC>(out + (t0 + i) * p.out_stride, o);
      }
      return;
    }
  }
  for (int i = 0; i < TOK; ++i) {
    const int64_t t = t0 + i;
    if (t >= p.tokens) return;
    const int64_t b = p.tok_seg ? p.tok_seg[t] : t;
    const int local = static_cast<int>(t - (p.seg_start ? p.seg_start[b] : t));
    const int pos = static_cast<int>(p.positions[t]);
    T* ring = state + p.slots[b] * taps * p.channels;
    float acc[VEC], newest[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) acc[j] = bias[j];
#pragma unroll
    for (int d = 0; d < (TAPS > 0 ? TAPS : taps); ++d) {
      if (d <= pos) {
        float v[VEC], w[VEC];
        if (d <= local) ldv<VEC>(x + (t - d) * p.x_stride, v);
        else ldv<VEC>(ring + static_cast<int64_t>((pos - d) % taps) * p.channels, v);
        ldv<VEC>(p.w + static_cast<int64_t>(d) * p.channels + c, w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          acc[j] += w[j] * v[j];
          if (d == 0) newest[j] = v[j];
        }
      }
    }
    float o[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = silu_f(acc[j]);
    stv<VEC>(out + t * p.out_stride, o);
    if (p.store) stv<VEC>(ring + static_cast<int64_t>(pos % taps) * p.channels, newest);
  }
}

constexpr int kConvTokens = 8;

template <typename T, int VEC>
void launch_conv(const ConvParams& p, bool decode, hipStream_t st) {
  const int tok = decode ? 1 : kConvTokens;
  const dim3 grid((p.channels + 256 * VEC - 1) / (256 * VEC), static_cast<unsigned>((p.tokens + tok - 1) / tok));
#define SGL_CONV(TAPS)                                                                                          \
  do {                                                                                                          \
    if (decode) hipLaunchKernelGGL((conv_silu_kernel<T, VEC, TAPS, 1>), grid, dim3(256), 0, st, p);             \
    else hipLaunchKernelGGL((conv_silu_kernel<T, VEC, TAPS, kConvTokens>), grid, dim3(256), 0, st, p);          \
  } while (0)
  switch (p.taps) {
    case 2: SGL_CONV(2); break;
    case 3: SGL_CONV(3); break;
    case 4: SGL_CONV(4); break;
    default: SGL_CONV(0);
  }
#undef SGL_CONV
}

// The last taps - 1 inputs of every segment into the ring (after conv_silu_kernel has read the ring).
template <typename T>
__global__ __launch_bounds__(256) void conv_state_kernel(ConvParams p, const int32_t* __restrict__ seg_len) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= p.channels) return;
  const int64_t b = blockIdx.y;
  const int64_t start = p.seg_start[b], n = seg_len[b];
  T* ring = static_cast<T*>(p.state) + p.slots[b] * p.taps * p.channels;
  for (int64_t i = n > p.taps - 1 ? n - (p.taps - 1) : 0; i < n; ++i)
    ring[(p.positions[start + i] % p.taps) * p.channels + c] = static_cast<const T*>(p.x)[(start + i) * p.x_stride + c];
}

// ---------------------------------------------------------------------------------------------------------------
// State tile of a step workgroup: 64 value columns (16 lanes of 4) x up to 16 * NR state rows (16 row groups), in registers.
constexpr int kStepCols = 64;

__device__ __forceinline__ void load_state4(const float* p, int ncol, bool vec, float (&s)[4]) {
  if (vec) { ld4(p, s); return; }
#pragma unroll
  for (int j = 0; j < 4; ++j) s[j] = j < ncol ? p[j] : 0.f;
}
__device__ __forceinline__ void store_state4(float* p, int ncol, bool vec, const float (&s)[4]) {
  if (vec) { st4(p, s); return; }
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (j < ncol) p[j] = s[j];
}

// sums of `K` values over the 16 row groups, for each of the 16 column lanes; `buf` is one of two alternating buffers
template <int K>
__device__ __forceinline__ void reduce_rows(float (&v)[K], float* buf) {
#pragma unroll
  for (int k = 0; k < K; ++k) {
    v[k] += __shfl_xor(v[k], 16, 64);
    v[k] += __shfl_xor(v[k], 32, 64);
  }
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  if (lane < 16) {
#pragma unroll
    for (int k = 0; k < K; ++k) buf[(wave * K + k) * 16 + lane] = v[k];
  }
  __syncthreads();
#pragma unroll
  for (int k = 0; k < K; ++k) {
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) s += buf[(w * K + k) * 16 + (lane & 15)];
    v[k] = s;
  }
}

struct Mamba2Params {
  const void* xbc;           // [tokens, inner + 2 * groups * N] convolved
  int64_t xbc_stride;
  const void* dt;            // [tokens, heads]
  int64_t dt_stride;
  const float *A_log, *dt_bias, *D;
  float* state;              // [slots, heads, N, P]
  const int64_t* slots;
  const int64_t* positions;
  const int32_t *seg_start, *seg_len;
  void* y;                   // [tokens, heads * P]
  int64_t y_stride;
  int heads, P, N, groups;
};

template <typename T, int NR>
__global__ __launch_bounds__(256) void mamba2_step_kernel(Mamba2Params p) {
  __shared__ float red[2][4 * 4 * 16];
  const int b = blockIdx.x, h = blockIdx.y;
  const int cl = threadIdx.x & 15, rg = threadIdx.x >> 4;
  const int col = blockIdx.z * kStepCols + cl * 4;
  const int ncol = p.P - col < 0 ? 0 : (p.P - col > 4 ? 4 : p.P - col);
  const bool vec = ncol == 4 && (p.P & 3) == 0;
  const int64_t t0 = p.seg_start ? p.seg_start[b] : b;
  const int len = p.seg_len ? p.seg_len[b] : 1;
  if (len <= 0) return;
  const int64_t pos0 = p.positions[t0];
  const int g = h / (p.heads / p.groups);
  float* S = p.state + (p.slots[b] * p.heads + h) * static_cast<int64_t>(p.N) * p.P + col;
  float s[NR][4];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int n = rg + 16 * i;
#pragma unroll
    for (int j = 0; j < 4; ++j) s[i][j] = 0.f;
    if (pos0 > 0 && n < p.N && ncol > 0) load_state4(S + static_cast<int64_t>(n) * p.P, ncol, vec, s[i]);
  }
  const float a = -expf(p.A_log[h]), dtb = p.dt_bias[h], dskip = p.D[h];
  const int inner = p.heads * p.P;
  for (int k = 0; k < len; ++k) {
    const int64_t t = t0 + k;
    const T* row = static_cast<const T*>(p.xbc) + t * p.xbc_stride;
    const float dt = softplus_f(ld1(static_cast<const T*>(p.dt) + t * p.dt_stride + h) + dtb);
    const float decay = expf(a * dt);
    float x[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) x[j] = j < ncol ? ld1(row + h * p.P + col + j) : 0.f;
    const T* B = row + inner + g * p.N;
    const T* C = B + p.groups * p.N;
    float y[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int n = rg + 16 * i;
      if (n < p.N) {
        const float bd = ld1(B + n) * dt, c = ld1(C + n);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          s[i][j] = s[i][j] * decay + bd * x[j];
          y[j] += s[i][j] * c;
        }
      }
    }
    reduce_rows<4>(y, red[k & 1]);
    if (rg == 0) {
      T* o = static_cast<T*>(p.y) + t * p.y_stride + h * p.P + col;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j < ncol) st1(o + j, y[j] + dskip * x[j]);
    }
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int n = rg + 16 * i;
    if (n < p.N && ncol > 0) store_state4(S + static_cast<int64_t>(n) * p.P, ncol, vec, s[i]);
  }
}

struct DeltaParams {
  const void* qkv;           // [tokens, 2 * kv_heads * K + heads * V] convolved: q | k | v
  int64_t qkv_stride;
  const void *b, *a;         // [tokens, heads]
  int64_t ba_stride;
  const float *A_log, *dt_bias;
  float* state;              // [slots, heads, K, V]
  const int64_t* slots;
  const int64_t* positions;
  const int32_t *seg_start, *seg_len;
  void* o;                   // [tokens, heads * V]
  int64_t o_stride;
  int heads, kv_heads, K, V;
  float q_scale;
};

// One token:  S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q  with unit k, q.  With r = (gS)^T k and
// w = (gS)^T q the read-out is o = w + (k . q) u, so one pass over the tile serves both contractions, and the squared
// lengths of k and q join the same row reduction (the contractions run on the raw vectors and are scaled afterwards).
template <typename T, int NR>
__global__ __launch_bounds__(256) void delta_step_kernel(DeltaParams p) {
  __shared__ float red[2][4 * 11 * 16];
  const int b = blockIdx.x, h = blockIdx.y;
  const int cl = threadIdx.x & 15, rg = threadIdx.x >> 4;
  const int col = blockIdx.z * kStepCols + cl * 4;
  const int ncol = p.V - col < 0 ? 0 : (p.V - col > 4 ? 4 : p.V - col);
  const bool vec = ncol == 4 && (p.V & 3) == 0;
  const int64_t t0 = p.seg_start ? p.seg_start[b] : b;
  const int len = p.seg_len ? p.seg_len[b] : 1;
  if (len <= 0) return;
  const int64_t pos0 = p.positions[t0];
  const int kh = h / (p.heads / p.kv_heads);
  float* S = p.state + (p.slots[b] * p.heads + h) * static_cast<int64_t>(p.K) * p.V + col;
  float s[NR][4];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int n = rg + 16 * i;
#pragma unroll
    for (int j = 0; j < 4; ++j) s[i][j] = 0.f;
    if (pos0 > 0 && n < p.K && ncol > 0) load_state4(S + static_cast<int64_t>(n) * p.V, ncol, vec, s[i]);
  }
  const float a = -expf(p.A_log[h]), dtb = p.dt_bias[h];
  for (int t_i = 0; t_i < len; ++t_i) {
    const int64_t t = t0 + t_i;
    const T* row = static_cast<const T*>(p.qkv) + t * p.qkv_stride;
    const T* qr = row + kh * p.K;
    const T* kr = qr + p.kv_heads * p.K;
    const T* vr = row + 2 * p.kv_heads * p.K + h * p.V + col;
    const float decay = expf(a * softplus_f(ld1(static_cast<const T*>(p.a) + t * p.ba_stride + h) + dtb));
    const float beta = sigmoid_f(ld1(static_cast<const T*>(p.b) + t * p.ba_stride + h));
    float kk[NR], acc[11];
#pragma unroll
    for (int j = 0; j < 11; ++j) acc[j] = 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int n = rg + 16 * i;
      kk[i] = 0.f;
      if (n < p.K) {
        kk[i] = ld1(kr + n);
        const float q = ld1(qr + n);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          s[i][j] *= decay;
          acc[j] += s[i][j] * kk[i];
          acc[4 + j] += s[i][j] * q;
        }
        acc[8] += kk[i] * kk[i];
        acc[9] += q * q;
        acc[10] += kk[i] * q;
      }
    }
    reduce_rows<11>(acc, red[t_i & 1]);
    const float ik = 1.0f / sqrtf(acc[8] + 1e-6f);
    const float iq = p.q_scale / sqrtf(acc[9] + 1e-6f);
    const float kq = acc[10] * ik * iq;
    float u[4], o[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      u[j] = j < ncol ? beta * (ld1(vr + j) - acc[j] * ik) : 0.f;
      o[j] = acc[4 + j] * iq + kq * u[j];
    }
#pragma unroll
    for (int i = 0; i < NR; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) s[i][j] += kk[i] * ik * u[j];
    if (rg == 0) {
      T* orow = static_cast<T*>(p.o) + t * p.o_stride + h * p.V + col;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j < ncol) st1(orow + j, o[j]);
    }
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int n = rg + 16 * i;
    if (n < p.K && ncol > 0) store_state4(S + static_cast<int64_t>(n) * p.V, ncol, vec, s[i]);
  }
}

struct MemoryParams {
  const void *q, *k, *v;     // [tokens, heads * D], [.., heads * D], [.., heads * V], columns of one row
  const void *gi, *gf;       // [tokens, heads] gates as projected
  int64_t stride;            // of all five
  const float *bi, *bf;      // [heads]
  float* state;              // [slots, heads, D, V], relative to e^m
  float* norm;               // [slots, heads, ceil(V / 16), D + 1]: the sum of the keys, then m; one copy per 16 value columns
  const int64_t* slots;
  const int64_t* positions;
  const int32_t *seg_start, *seg_len;
  void* o;                   // [tokens, heads * V]
  int64_t o_stride;
  int heads, D, V, blocks;
  float cap, q_scale;
};

// One token, with log gates i = cap tanh((gi + bi) / cap), f = log sigmoid(cap tanh((gf + bf) / cap)) and a running maximum m:
//   m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T, n alike with k alone;  o = S^T q / (max(|n.q|, e^-m') + 1e-6)
// n and m belong to the whole head: every workgroup keeps them for itself, in the copies of its own columns, so that none reads
// what another one writes.
template <typename T, int NR>
__global__ __launch_bounds__(256) void memory_step_kernel(MemoryParams p) {
  __shared__ float red[2][4 * 5 * 16];
  const int b = blockIdx.x, h = blockIdx.y;
  const int cl = threadIdx.x & 15, rg = threadIdx.x >> 4;
  const int col = blockIdx.z * kStepCols + cl * 4;
  const int ncol = p.V - col < 0 ? 0 : (p.V - col > 4 ? 4 : p.V - col);
  const bool vec = ncol == 4 && (p.V & 3) == 0;
  const int64_t t0 = p.seg_start ? p.seg_start[b] : b;
  const int len = p.seg_len ? p.seg_len[b] : 1;
  if (len <= 0) return;
  const int64_t pos0 = p.positions[t0], head = p.slots[b] * p.heads + h;
  const int block = blockIdx.z * (kStepCols / 16);
  float* S = p.state + head * p.D * p.V + col;
  float* norm = p.norm + (head * p.blocks + block) * (p.D + 1);
  float s[NR][4], n[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int r = rg + 16 * i;
    n[i] = pos0 > 0 && r < p.D ? norm[r] : 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) s[i][j] = 0.f;
    if (pos0 > 0 && r < p.D && ncol > 0) load_state4(S + static_cast<int64_t>(r) * p.V, ncol, vec, s[i]);
  }
  float m = pos0 > 0 ? norm[p.D] : 0.f;
  const float bi = p.bi[h], bf = p.bf[h];
  for (int u = 0; u < len; ++u) {
    const int64_t t = t0 + u, row = t * p.stride;
    const T* qr = static_cast<const T*>(p.q) + row + h * p.D;
    const T* kr = static_cast<const T*>(p.k) + row + h * p.D;
    const T* vr = static_cast<const T*>(p.v) + row + h * p.V + col;
    const float gi = p.cap * tanhf((ld1(static_cast<const T*>(p.gi) + row + h) + bi) / p.cap);
    const float gf = -softplus_f(-p.cap * tanhf((ld1(static_cast<const T*>(p.gf) + row + h) + bf) / p.cap));
    const float top = fmaxf(gf + m, gi), keep = expf(gf + m - top), add = expf(gi - top);
    m = top;
    float v[4], acc[5] = {0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = j < ncol ? ld1(vr + j) : 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int r = rg + 16 * i;
      if (r < p.D) {
        const float k = ld1(kr + r) * add, q = ld1(qr + r) * p.q_scale;
        n[i] = n[i] * keep + k;
        acc[4] += n[i] * q;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          s[i][j] = s[i][j] * keep + k * v[j];
          acc[j] += s[i][j] * q;
        }
      }
    }
    reduce_rows<5>(acc, red[u & 1]);
    if (rg == 0) {
      const float inv = 1.0f / (fmaxf(fabsf(acc[4]), expf(-m)) + 1e-6f);
      T* o = static_cast<T*>(p.o) + t * p.o_stride + h * p.V + col;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j < ncol) st1(o + j, acc[j] * inv);
    }
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int r = rg + 16 * i;
    if (r >= p.D) continue;
    if (ncol > 0) store_state4(S + static_cast<int64_t>(r) * p.V, ncol, vec, s[i]);
    if (cl < kStepCols / 16 && block + cl < p.blocks) norm[cl * (p.D + 1) + r] = n[i];
  }
  if (rg == 0 && cl < kStepCols / 16 && block + cl < p.blocks) norm[cl * (p.D + 1) + p.D] = m;
}

template <typename T>
void launch_memory(const MemoryParams& p, int segs, hipStream_t st) {
  const dim3 grid(segs, p.heads, (p.V + kStepCols - 1) / kStepCols);
  const int nr = (p.D + 15) / 16;
  if (nr <= 2) hipLaunchKernelGGL((memory_step_kernel<T, 2>), grid, dim3(256), 0, st, p);
  else if (nr <= 4) hipLaunchKernelGGL((memory_step_kernel<T, 4>), grid, dim3(256), 0, st, p);
  else if (nr <= 8) hipLaunchKernelGGL((memory_step_kernel<T, 8>), grid, dim3(256), 0, st, p);
  else if (nr <= 16) hipLaunchKernelGGL((memory_step_kernel<T, 16>), grid, dim3(256), 0, st, p);
  else hipLaunchKernelGGL((memory_step_kernel<T, 32>), grid, dim3(256), 0, st, p);
}

// ---------------------------------------------------------------------------------------------------------------
struct ShiftParams {
  const void* h;             // [tokens, width]
  int64_t h_stride;
  const float* mu;           // [width]
  void* state;               // [slots, width]: the last row of every request
  const int64_t* slots;
  const int64_t* positions;
  const int32_t *tok_seg, *seg_start, *seg_len;
  void* out;                 // not h
  int64_t out_stride;
  int64_t tokens;
  int width;
};

constexpr int kShiftTokens = 4;

// out[t] = h[t] + (h in front of t - h[t]) * mu.  A thread owns VEC columns of a few tokens; the one that owns a segment's first token
// reads what the request left and then leaves the segment's last row, so nothing is read behind its own replacement.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void token_shift_kernel(ShiftParams p) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (c >= p.width) return;
  const T* h = static_cast<const T*>(p.h) + c;
  const int64_t t0 = static_cast<int64_t>(blockIdx.y) * kShiftTokens;
  float mu[VEC], v[kShiftTokens + 1][VEC];
  ldv<VEC>(p.mu + c, mu);
#pragma unroll
  for (int i = 0; i <= kShiftTokens; ++i) {            // (rows outside the batch are not used)
    int64_t t = t0 + i - 1;
    t = t < 0 ? 0 : t >= p.tokens ? p.tokens - 1 : t;
    ldv<VEC>(h + t * p.h_stride, v[i]);
  }
#pragma unroll
  for (int i = 0; i < kShiftTokens; ++i) {
    const int64_t t = t0 + i;
    if (t >= p.tokens) return;
    const int64_t b = p.tok_seg[t], start = p.seg_start[b];
    float o[VEC];
    if (t == start) {
      T* left = static_cast<T*>(p.state) + p.slots[b] * p.width + c;
      float front[VEC], last[VEC];
      ldv<VEC>(left, front);
      ldv<VEC>(h + (start + p.seg_len[b] - 1) * p.h_stride, last);
      const bool fresh = p.positions[t] <= 0;
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = v[i + 1][j] + ((fresh ? 0.f : front[j]) - v[i + 1][j]) * mu[j];
      stv<VEC>(left, last);
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = v[i + 1][j] + (v[i][j] - v[i + 1][j]) * mu[j];
    }
    stv<VEC>(static_cast<T*>(p.out) + t * p.out_stride + c, o);
  }
}

template <typename T, int VEC>
void launch_shift(const ShiftParams& p, hipStream_t st) {
  const dim3 grid((p.width + 256 * VEC - 1) / (256 * VEC), static_cast<unsigned>((p.tokens + kShiftTokens - 1) / kShiftTokens));
  hipLaunchKernelGGL((token_shift_kernel<T, VEC>), grid, dim3(256), 0, st, p);
}

template <typename T>
int launch_mamba2(const Mamba2Params& p, int segs, hipStream_t st) {
  const dim3 grid(segs, p.heads, (p.P + kStepCols - 1) / kStepCols);
  const int nr = (p.N + 15) / 16;
  if (nr <= 2) hipLaunchKernelGGL((mamba2_step_kernel<T, 2>), grid, dim3(256), 0, st, p);
  else if (nr <= 4) hipLaunchKernelGGL((mamba2_step_kernel<T, 4>), grid, dim3(256), 0, st, p);
  else if (nr <= 8) hipLaunchKernelGGL((mamba2_step_kernel<T, 8>), grid, dim3(256), 0, st, p);
  else if (nr <= 16) hipLaunchKernelGGL((mamba2_step_kernel<T, 16>), grid, dim3(256), 0, st, p);
  else hipLaunchKernelGGL((mamba2_step_kernel<T, 32>), grid, dim3(256), 0, st, p);
  return 0;
}

template <typename T>
int launch_delta(const DeltaParams& p, int segs, hipStream_t st) {
  const dim3 grid(segs, p.heads, (p.V + kStepCols - 1) / kStepCols);
  const int nr = (p.K + 15) / 16;
  if (nr <= 2) hipLaunchKernelGGL((delta_step_kernel<T, 2>), grid, dim3(256), 0, st, p);
  else if (nr <= 4) hipLaunchKernelGGL((delta_step_kernel<T, 4>), grid, dim3(256), 0, st, p);
  else if (nr <= 8) hipLaunchKernelGGL((delta_step_kernel<T, 8>), grid, dim3(256), 0, st, p);
  else if (nr <= 16) hipLaunchKernelGGL((delta_step_kernel<T, 16>), grid, dim3(256), 0, st, p);
  else hipLaunchKernelGGL((delta_step_kernel<T, 32>), grid, dim3(256), 0, st, p);
  return 0;
}

}  // namespace

extern "C" {

int sgl_amd_causal_conv_silu(int is_f32, const void* x, int64_t x_stride, const float* weight, const float* bias, void* state,
                             const int64_t* slots, const int64_t* positions, const int32_t* tok_seg, const int32_t* seg_start,
                             const int32_t* seg_len, void* out, int64_t out_stride, int64_t tokens, int segments, int channels,
                             int taps, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(x && weight && state && slots && positions && out && channels > 0 && taps > 0, "causal_conv_silu: null operand");
  SGL_CHECK_ARG((tok_seg && seg_start && seg_len) || (!tok_seg && !seg_start && !seg_len && tokens == segments),
                "causal_conv_silu: segment arrays come together, or one token per request");
  if (tokens <= 0) return 0;
  SGL_CHECK_ARG((tok_seg ? (tokens + kConvTokens - 1) / kConvTokens : tokens) <= 65535 && segments <= 65535, "causal_conv_silu: %lld tokens", (long long)tokens);
  const bool decode = tok_seg == nullptr;
  ConvParams p{x, x_stride, weight, bias, state, slots, positions, tok_seg, seg_start, out, out_stride, tokens, channels, taps, decode ? 1 : 0};
  const size_t a = is_f32 ? 16 : 8;
  const bool vec = channels % 4 == 0 && x_stride % 4 == 0 && out_stride % 4 == 0 && aligned_to(x, a) && aligned_to(out, a) &&
                   aligned_to(state, a) && aligned_to(weight, 16) && aligned_to(bias, 16);
  hipStream_t st = as_stream(stream);
  if (is_f32) vec ? launch_conv<float, 4>(p, decode, st) : launch_conv<float, 1>(p, decode, st);
  else vec ? launch_conv<uint16_t, 4>(p, decode, st) : launch_conv<uint16_t, 1>(p, decode, st);
  if (!decode && taps > 1) {
    const dim3 sg((channels + 255) / 256, segments);
    if (is_f32) hipLaunchKernelGGL((conv_state_kernel<float>), sg, dim3(256), 0, st, p, seg_len);
    else hipLaunchKernelGGL((conv_state_kernel<uint16_t>), sg, dim3(256), 0, st, p, seg_len);
  }
  SGL_CHECK_LAUNCH("causal_conv_silu");
  return 0;
}

int sgl_amd_mamba2_step(int is_f32, const void* xbc, int64_t xbc_stride, const void* dt, int64_t dt_stride, const float* A_log,
                        const float* dt_bias, const float* D, float* state, const int64_t* slots, const int64_t* positions,
                        const int32_t* seg_start, const int32_t* seg_len, void* y, int64_t y_stride, int segments, int heads, int head_dim,
                        int state_dim, int groups, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(xbc && dt && A_log && dt_bias && D && state && slots && positions && y, "mamba2_step: null operand");
  SGL_CHECK_ARG(groups > 0 && heads > 0 && heads % groups == 0 && heads <= 65535 && head_dim > 0 && state_dim > 0 && state_dim <= 512,
                "mamba2_step: %d heads in %d groups, state %d (at most 512)", heads, groups, state_dim);
  SGL_CHECK_ARG((seg_start == nullptr) == (seg_len == nullptr), "mamba2_step: segment arrays come together");
  if (segments <= 0) return 0;
  Mamba2Params p{xbc, xbc_stride, dt, dt_stride, A_log, dt_bias, D, state, slots, positions, seg_start, seg_len, y, y_stride,
                 heads, head_dim, state_dim, groups};
  if (is_f32) launch_mamba2<float>(p, segments, as_stream(stream));
  else launch_mamba2<uint16_t>(p, segments, as_stream(stream));
  SGL_CHECK_LAUNCH("mamba2_step");
  return 0;
}

int sgl_amd_delta_step(int is_f32, const void* qkv, int64_t qkv_stride, const void* b, const void* a, int64_t ba_stride,
                       const float* A_log, const float* dt_bias, float* state, const int64_t* slots, const int64_t* positions,
                       const int32_t* seg_start, const int32_t* seg_len, void* o, int64_t o_stride, int segments, int heads, int kv_heads,
                       int key_dim, int value_dim, float q_scale, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(qkv && b && a && A_log && dt_bias && state && slots && positions && o, "delta_step: null operand");
  SGL_CHECK_ARG(kv_heads > 0 && heads > 0 && heads % kv_heads == 0 && heads <= 65535 && value_dim > 0 && key_dim > 0 && key_dim <= 512,
                "delta_step: %d value heads over %d key heads, key dim %d (at most 512)", heads, kv_heads, key_dim);
  SGL_CHECK_ARG((seg_start == nullptr) == (seg_len == nullptr), "delta_step: segment arrays come together");
  if (segments <= 0) return 0;
  DeltaParams p{qkv, qkv_stride, b, a, ba_stride, A_log, dt_bias, state, slots, positions, seg_start, seg_len, o, o_stride,
                heads, kv_heads, key_dim, value_dim, q_scale};
  if (is_f32) launch_delta<float>(p, segments, as_stream(stream));
  else launch_delta<uint16_t>(p, segments, as_stream(stream));
  SGL_CHECK_LAUNCH("delta_step");
  return 0;
}

int sgl_amd_memory_step(int is_f32, const void* q, const void* k, const void* v, const void* gate_i, const void* gate_f, int64_t stride,
                        const float* bias_i, const float* bias_f, float* state, float* norm, const int64_t* slots, const int64_t* positions,
                        const int32_t* seg_start, const int32_t* seg_len, void* o, int64_t o_stride, int segments, int heads, int key_dim,
                        int value_dim, float gate_cap, float q_scale, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(q && k && v && gate_i && gate_f && bias_i && bias_f && state && norm && slots && positions && o, "memory_step: null operand");
  SGL_CHECK_ARG(heads > 0 && heads <= 65535 && value_dim > 0 && key_dim > 0 && key_dim <= 512 && gate_cap > 0.f,
                "memory_step: %d heads of %d x %d (keys at most 512), gate cap %g", heads, key_dim, value_dim, gate_cap);
  SGL_CHECK_ARG((seg_start == nullptr) == (seg_len == nullptr), "memory_step: segment arrays come together");
  if (segments <= 0) return 0;
  MemoryParams p{q, k, v, gate_i, gate_f, stride, bias_i, bias_f, state, norm, slots, positions, seg_start, seg_len, o, o_stride,
                 heads, key_dim, value_dim, (value_dim + 15) / 16, gate_cap, q_scale};
  if (is_f32) launch_memory<float>(p, segments, as_stream(stream));
  else launch_memory<uint16_t>(p, segments, as_stream(stream));
  SGL_CHECK_LAUNCH("memory_step");
  return 0;
}

int sgl_amd_token_shift(int is_f32, const void* h, int64_t h_stride, const float* mu, void* state, const int64_t* slots, const int64_t* positions,
                        const int32_t* tok_seg, const int32_t* seg_start, const int32_t* seg_len, void* out, int64_t out_stride, int64_t tokens,
                        int width, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(h && mu && state && slots && positions && tok_seg && seg_start && seg_len && out && h != out && width > 0, "token_shift: null operand, or in place");
  if (tokens <= 0) return 0;
  SGL_CHECK_ARG((tokens + kShiftTokens - 1) / kShiftTokens <= 65535, "token_shift: %lld tokens", (long long)tokens);
  ShiftParams p{h, h_stride, mu, state, slots, positions, tok_seg, seg_start, seg_len, out, out_stride, tokens, width};
  const bool vec = width % 8 == 0 && h_stride % 8 == 0 && out_stride % 8 == 0 && aligned_to(h, 16) && aligned_to(out, 16) && aligned_to(state, 16) &&
                   aligned_to(mu, 16);
  hipStream_t st = as_stream(stream);
  if (is_f32) vec ? launch_shift<float, 8>(p, st) : launch_shift<float, 1>(p, st);
  else vec ? launch_shift<uint16_t, 8>(p, st) : launch_shift<uint16_t, 1>(p, st);
  SGL_CHECK_LAUNCH("token_shift");
  return 0;
}

}  // extern "C"
