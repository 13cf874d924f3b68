// Mamba-2, gated-delta-rule and matrix-memory state updates in chunks of 32 tokens, for prefill-sized segments.
//
// A workgroup owns one (segment, head) and up to 64 value columns (a wave = 16 of them) and walks the segment; the state tile
// stays in the accumulators of v_mfma_f32_16x16x4_f32 for the whole walk.  Everything is fp32: operands are widened when they
// are staged, so the recurrence sees no 16-bit rounding beyond its inputs', and bf16 and fp32 models share one body.
//
// Register k-order.  The matrix instruction contracts over four slots g = lane / 16.  An accumulator tile holds row
// 4 g + r in register r, so feeding register r of tile t as the B operand pairs slot g with row 16 t + 4 g + r; the A operand is
// read in that order (four consecutive floats per lane serve four instructions).  State, corrected values and read-outs thus
// go from one product into the next without leaving their registers.
//
// With c_i = sum of the log decays up to token i of the chunk (kept in double: differences of far larger sums stay exact),
//   Mamba-2:  y_i = e^{c_i} S0^T C_i + sum_{j<=i} e^{c_i-c_j} dt_j (C_i.B_j) x_j + D x_i
//             S   = e^{c_n} S0 + sum_j e^{c_n-c_j} dt_j B_j x_j^T
//   delta:    (I + A) U = beta (v - e^{c_i} S0^T k_i),  A_ij = beta_i e^{c_i-c_j} (k_i.k_j) for j < i
//             o_i = e^{c_i} S0^T q_i + sum_{j<=i} e^{c_i-c_j} (q_i.k_j) u_j
//             S   = e^{c_n} S0 + sum_j e^{c_n-c_j} k_j u_j^T
//   memory:   with a_j = i_j - c_j and g_i = max(m0, a_1 .. a_i), so that c_i + g_i is the running maximum behind token i,
//             (y | d)_i = e^{m0-g_i} (S0 | n0)^T q_i + sum_{j<=i} e^{a_j-g_i} (q_i.k_j) (v_j | 1),  o_i = y_i / (max(|d_i|, e^{-c_i-g_i}) + 1e-6)
//             (S | n) = e^{m0-g_n} (S0 | n0) + sum_j e^{a_j-g_n} k_j (v_j | 1)^T,  m = c_n + g_n
// (I + A)^-1 is formed by forward substitution in 16-token blocks, which stays accurate for repeated keys.
#include "elem_io.hpp"
#include "sglang_amd.h"

using namespace sgl_amd;

namespace {

constexpr int kQ = 32;            // tokens per chunk
constexpr int kSq = kQ + 4;       // row stride of the 32 x 32 matrices (4 mod 16 floats: conflict-free in both access patterns)

__device__ __forceinline__ f32x4_t mfma4(float a, float b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// rows [0, 32) x [0, n) of a strided activation matrix on their way to LDS (row stride `ls`): fetched into registers a chunk ahead,
// widened when they are committed; rows >= len and columns n .. NP are zero.  256 threads, four elements a piece.
template <typename T> struct Raw4;
template <> struct Raw4<uint16_t> { uint2 v; };
template <> struct Raw4<float> { f32x4_t v; };

template <typename T, int NP>
struct RowTile {
  static constexpr int kPieces = NP / 32;            // kQ * NP / 4 / 256
  Raw4<T> raw[kPieces];

  __device__ __forceinline__ void fetch(const T* src, int64_t stride, int len, int n, bool vec) {
#pragma unroll
    for (int i = 0; i < kPieces; ++i) {
      const int idx = i * 256 + threadIdx.x, row = idx / (NP / 4), c = (idx % (NP / 4)) * 4;
      raw[i] = Raw4<T>{};
      if (row < len && c < n) {
        const T* a = src + row * stride + c;
        if (vec) {
          raw[i] = *reinterpret_cast<const Raw4<T>*>(a);
        } else {
          T* e = reinterpret_cast<T*>(&raw[i]);
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (c + j < n) e[j] = a[j];
        }
      }
    }
  }
  __device__ __forceinline__ void commit(float* dst, int ls) const {
#pragma unroll
    for (int i = 0; i < kPieces; ++i) {
      const int idx = i * 256 + threadIdx.x, row = idx / (NP / 4), c = (idx % (NP / 4)) * 4;
      float f[4];
      ld4(reinterpret_cast<const T*>(&raw[i]), f);
      *reinterpret_cast<f32x4_t*>(dst + row * ls + c) = f32x4_t{f[0], f[1], f[2], f[3]};
    }
  }
};

// inclusive prefix sum over 32 lanes of a wave, in double
__device__ __forceinline__ double scan32(double v, int lane) {
#pragma unroll
  for (int off = 1; off < kQ; off <<= 1) {
    const double u = __shfl_up(v, off, 64);
    if (lane >= off) v += u;
  }
  return v;
}

// 16 x 16 tile of X Y^T over npad columns, rows of X from xi, rows of Y from yj (both LDS, stride ls)
__device__ __forceinline__ f32x4_t gram_tile(const float* x, const float* y, int npad, int ls, int i16, int g) {
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
  const float* xr = x + i16 * ls + 4 * g;
  const float* yr = y + i16 * ls + 4 * g;
  for (int t = 0; t < npad; t += 16) {
    const f32x4_t a = *reinterpret_cast<const f32x4_t*>(xr + t), b = *reinterpret_cast<const f32x4_t*>(yr + t);
#pragma unroll
    for (int r = 0; r < 4; ++r) acc = mfma4(a[r], b[r], acc);
  }
  return acc;
}

struct Mamba2ChunkParams {
  const void* xbc;
  int64_t xbc_stride;
  const void* dt;
  int64_t dt_stride;
  const float *A_log, *dt_bias, *D;
  float* state;
  const int64_t* slots;
  const int64_t* positions;
  const int32_t *seg_start, *seg_len;
  void* y;
  int64_t y_stride;
  int heads, P, N, groups, vec, col_waves;
};

template <typename T, int NT>
__global__ __launch_bounds__(256, NT <= 8 ? 2 : 1) void mamba2_chunk_kernel(Mamba2ChunkParams p) {
  constexpr int NP = NT * 16, LS = NP + 4;
  __shared__ __attribute__((aligned(16))) float Bs[kQ * LS];
  __shared__ __attribute__((aligned(16))) float Cs[kQ * LS];
  __shared__ __attribute__((aligned(16))) float Gs[kQ * kSq];
  __shared__ double cum[kQ];
  __shared__ float dts[kQ];
  const int b = blockIdx.y, h = blockIdx.x;
  constexpr int waves = 4;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int col = (blockIdx.z * p.col_waves + wave) * 16 + i16;
  const bool live = wave < p.col_waves && col < p.P;           // waves without columns only help with the shared matrices
  const int64_t t0 = p.seg_start[b];
  const int total = p.seg_len[b];
  if (total <= 0) return;
  const int64_t pos0 = p.positions[t0];
  const int grp = h / (p.heads / p.groups), inner = p.heads * p.P;
  float* S = p.state + (p.slots[b] * p.heads + h) * static_cast<int64_t>(p.N) * p.P + col;
  f32x4_t s[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = 16 * t + 4 * g + r;
      s[t][r] = pos0 > 0 && live && n < p.N ? S[static_cast<int64_t>(n) * p.P] : 0.f;
    }
  const float a = -expf(p.A_log[h]), dtb = p.dt_bias[h], dskip = p.D[h];
  const T* xbc = static_cast<const T*>(p.xbc) + t0 * p.xbc_stride;
  const T* dtp = static_cast<const T*>(p.dt) + t0 * p.dt_stride + h;
  T* yp = static_cast<T*>(p.y) + t0 * p.y_stride + h * p.P + col;

  RowTile<T, NP> bt, ct;
  T xr[2][4], dtr = T{};
  auto fetch = [&](int c0) __attribute__((always_inline)) {
    const int len = total - c0 < kQ ? total - c0 : kQ;
    const T* rows = xbc + static_cast<int64_t>(c0) * p.xbc_stride;
    bt.fetch(rows + inner + grp * p.N, p.xbc_stride, len, p.N, p.vec);
    ct.fetch(rows + inner + (p.groups + grp) * p.N, p.xbc_stride, len, p.N, p.vec);
    // this wave's columns of x, token 16 tj + 4 g + r in [tj][r]
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * tj + 4 * g + r;
        xr[tj][r] = live && j < len ? rows[j * p.xbc_stride + h * p.P + col] : T{};
      }
    if (wave == 0 && lane < len) dtr = dtp[static_cast<int64_t>(c0 + lane) * p.dt_stride];
  };
  fetch(0);
  for (int c0 = 0; c0 < total; c0 += kQ) {
    const int len = total - c0 < kQ ? total - c0 : kQ;
    bt.commit(Bs, LS);
    ct.commit(Cs, LS);
    if (wave == 0) {
      const float dt = lane < len ? softplus_f(ld1(&dtr) + dtb) : 0.f;
      const double c = scan32(static_cast<double>(a * dt), lane);
      if (lane < kQ) { cum[lane] = c; dts[lane] = dt; }
    }
    float x[2][4];
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) x[tj][r] = ld1(&xr[tj][r]);
    __syncthreads();
    if (c0 + kQ < total) fetch(c0 + kQ);
    for (int tile = wave; tile < 3; tile += waves) {
      const int ti = tile > 0, tj = tile > 1;
      const f32x4_t gm = gram_tile(Cs + 16 * ti * LS, Bs + 16 * tj * LS, NP, LS, i16, g);
      const int j = 16 * tj + i16;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * ti + 4 * g + r;
        Gs[i * kSq + j] = j <= i ? gm[r] * expf(static_cast<float>(cum[i] - cum[j])) * dts[j] : 0.f;
      }
    }
    f32x4_t y[2];
#pragma unroll
    for (int ti = 0; ti < 2; ++ti) {
      y[ti] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const f32x4_t c = *reinterpret_cast<const f32x4_t*>(Cs + (16 * ti + i16) * LS + 16 * t + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) y[ti] = mfma4(c[r], s[t][r], y[ti]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) y[ti][r] *= expf(static_cast<float>(cum[16 * ti + 4 * g + r]));
    }
    __syncthreads();
#pragma unroll
    for (int ti = 0; ti < 2; ++ti)
#pragma unroll
      for (int tj = 0; tj <= ti; ++tj) {
        const f32x4_t w = *reinterpret_cast<const f32x4_t*>(Gs + (16 * ti + i16) * kSq + 16 * tj + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) y[ti] = mfma4(w[r], x[tj][r], y[ti]);
      }
#pragma unroll
    for (int ti = 0; ti < 2; ++ti)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * ti + 4 * g + r;
        if (live && i < len) st1(yp + static_cast<int64_t>(c0 + i) * p.y_stride, y[ti][r] + dskip * x[ti][r]);
      }
    const double cn = cum[kQ - 1];
    const float fix = expf(static_cast<float>(cn));
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * tj + 4 * g + r;
        x[tj][r] *= expf(static_cast<float>(cn - cum[j])) * dts[j];
      }
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      s[t] *= fix;
#pragma unroll
      for (int tj = 0; tj < 2; ++tj)
#pragma unroll
        for (int r = 0; r < 4; ++r) s[t] = mfma4(Bs[(16 * tj + 4 * g + r) * LS + 16 * t + i16], x[tj][r], s[t]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = 16 * t + 4 * g + r;
      if (live && n < p.N) S[static_cast<int64_t>(n) * p.P] = s[t][r];
    }
}

struct DeltaChunkParams {
  const void* qkv;
  int64_t qkv_stride;
  const void *b, *a;
  int64_t ba_stride;
  const float *A_log, *dt_bias;
  float* state;
  const int64_t* slots;
  const int64_t* positions;
  const int32_t *seg_start, *seg_len;
  void* o;
  int64_t o_stride;
  int heads, kv_heads, K, V, vec, col_waves;
  float q_scale;
};

template <typename T, int NT>
__global__ __launch_bounds__(256, NT <= 8 ? 2 : 1) void delta_chunk_kernel(DeltaChunkParams p) {
  constexpr int NP = NT * 16, LS = NP + 4;
  __shared__ __attribute__((aligned(16))) float Ks[kQ * LS];
  __shared__ __attribute__((aligned(16))) float Qs[kQ * LS];
  __shared__ __attribute__((aligned(16))) float As[kQ * kSq];   // A, then (I + A)^-1
  __shared__ __attribute__((aligned(16))) float Ps[kQ * kSq];
  __shared__ double cum[kQ];
  __shared__ float beta[kQ], ik[kQ], iq[kQ];
  const int b = blockIdx.y, h = blockIdx.x;
  constexpr int waves = 4;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int col = (blockIdx.z * p.col_waves + wave) * 16 + i16;
  const bool live = wave < p.col_waves && col < p.V;           // waves without columns only help with the shared matrices
  const int64_t t0 = p.seg_start[b];
  const int total = p.seg_len[b];
  if (total <= 0) return;
  const int64_t pos0 = p.positions[t0];
  const int kh = h / (p.heads / p.kv_heads);
  float* S = p.state + (p.slots[b] * p.heads + h) * static_cast<int64_t>(p.K) * p.V + col;
  f32x4_t s[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = 16 * t + 4 * g + r;
      s[t][r] = pos0 > 0 && live && n < p.K ? S[static_cast<int64_t>(n) * p.V] : 0.f;
    }
  const float a = -expf(p.A_log[h]), dtb = p.dt_bias[h];
  const T* qkv = static_cast<const T*>(p.qkv) + t0 * p.qkv_stride;
  const T* bp = static_cast<const T*>(p.b) + t0 * p.ba_stride + h;
  const T* ap = static_cast<const T*>(p.a) + t0 * p.ba_stride + h;
  T* op = static_cast<T*>(p.o) + t0 * p.o_stride + h * p.V + col;

  RowTile<T, NP> qt, kt;
  T vr[2][4], ar = T{}, br = T{};
  auto fetch = [&](int c0) __attribute__((always_inline)) {
    const int len = total - c0 < kQ ? total - c0 : kQ;
    const T* rows = qkv + static_cast<int64_t>(c0) * p.qkv_stride;
    qt.fetch(rows + kh * p.K, p.qkv_stride, len, p.K, p.vec);
    kt.fetch(rows + (p.kv_heads + kh) * p.K, p.qkv_stride, len, p.K, p.vec);
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * tj + 4 * g + r;
        vr[tj][r] = live && j < len ? rows[j * p.qkv_stride + 2 * p.kv_heads * p.K + h * p.V + col] : T{};
      }
    if (wave == 0 && lane < len) {
      ar = ap[static_cast<int64_t>(c0 + lane) * p.ba_stride];
      br = bp[static_cast<int64_t>(c0 + lane) * p.ba_stride];
    }
  };
  fetch(0);
  for (int c0 = 0; c0 < total; c0 += kQ) {
    const int len = total - c0 < kQ ? total - c0 : kQ;
    qt.commit(Qs, LS);
    kt.commit(Ks, LS);
    if (wave == 0) {
      const float lg = lane < len ? a * softplus_f(ld1(&ar) + dtb) : 0.f;
      const float bt = lane < len ? sigmoid_f(ld1(&br)) : 0.f;
      const double c = scan32(static_cast<double>(lg), lane);
      if (lane < kQ) { cum[lane] = c; beta[lane] = bt; }
    }
    f32x4_t u[2];       // v, then the right-hand side, then U
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) u[tj][r] = ld1(&vr[tj][r]);
    __syncthreads();
    if (c0 + kQ < total) fetch(c0 + kQ);
    // lengths of the 32 keys and queries: 8 lanes per vector
#pragma unroll
    for (int i = threadIdx.x >> 3; i < 2 * kQ; i += 32) {
      const float* v = (i < kQ ? Ks : Qs) + (i & (kQ - 1)) * LS;
      float ss = 0.f;
      for (int c = (threadIdx.x & 7) * 4; c < NP; c += 32) {
        const f32x4_t f = *reinterpret_cast<const f32x4_t*>(v + c);
        ss += f[0] * f[0] + f[1] * f[1] + f[2] * f[2] + f[3] * f[3];
      }
      ss += __shfl_xor(ss, 1, 64);
      ss += __shfl_xor(ss, 2, 64);
      ss += __shfl_xor(ss, 4, 64);
      if ((threadIdx.x & 7) == 0) {
        if (i < kQ) ik[i] = 1.0f / sqrtf(ss + 1e-6f);
        else iq[i - kQ] = p.q_scale / sqrtf(ss + 1e-6f);
      }
    }
    __syncthreads();
    // A first (the inversion waits for it), then the attention-like matrix of the read-out
    for (int tile = wave; tile < 3; tile += waves) {
      const int ti = tile > 0, tj = tile > 1;
      const f32x4_t gm = gram_tile(Ks + 16 * ti * LS, Ks + 16 * tj * LS, NP, LS, i16, g);
      const int j = 16 * tj + i16;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * ti + 4 * g + r;
        As[i * kSq + j] = j < i ? gm[r] * expf(static_cast<float>(cum[i] - cum[j])) * beta[i] * ik[i] * ik[j] : 0.f;
      }
    }
    __syncthreads();
    if (wave == waves - 1) {
      // The two 16 x 16 diagonal blocks of (I + A)^-1 side by side: lane = column, x_i = [i == column] - sum_{j < i} A_ij x_j,
      // two rows at a time; then the block below them is -X22 A21 X11, two small products.
      int blk = ((lane >> 4) & 1) * (16 * kSq + 16);
      float x[16];
#pragma unroll
      for (int i0 = 0; i0 < 16; i0 += 2) {
        f32x4_t w[2][4];
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
          for (int j = 0; j <= i0 + 1; j += 4) w[i][j / 4] = *reinterpret_cast<const f32x4_t*>(As + blk + (i0 + i) * kSq + j);
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          float acc[2] = {i0 + i == i16 ? 1.f : 0.f, 0.f};
#pragma unroll
          for (int j = 0; j < i0 + i; ++j) acc[j & 1] -= w[i][j / 4][j & 3] * x[j];
          x[i0 + i] = acc[0] + acc[1];
        }
        asm volatile("" : "+v"(blk) : "v"(x[i0 + 1]));   // the next rows are loaded behind these: 32 registers, not 160
      }
      if (lane < kQ) {
#pragma unroll
        for (int i = 0; i < 16; ++i) As[blk + i * kSq + i16] = x[i];
      }
      // (one wave: its LDS accesses complete in order)
      f32x4_t m = {0.f, 0.f, 0.f, 0.f}, x21 = {0.f, 0.f, 0.f, 0.f};
      const f32x4_t a21 = *reinterpret_cast<const f32x4_t*>(As + (16 + i16) * kSq + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) m = mfma4(a21[r], As[(4 * g + r) * kSq + i16], m);
      const f32x4_t x22 = *reinterpret_cast<const f32x4_t*>(As + (16 + i16) * kSq + 16 + 4 * g);
#pragma unroll
      for (int r = 0; r < 4; ++r) x21 = mfma4(-x22[r], m[r], x21);
#pragma unroll
      for (int r = 0; r < 4; ++r) As[(16 + 4 * g + r) * kSq + i16] = x21[r];
    }
    for (int tile = wave; tile < 3; tile += waves) {
      const int ti = tile > 0, tj = tile > 1;
      const f32x4_t gm = gram_tile(Qs + 16 * ti * LS, Ks + 16 * tj * LS, NP, LS, i16, g);
      const int j = 16 * tj + i16;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * ti + 4 * g + r;
        Ps[i * kSq + j] = j <= i ? gm[r] * expf(static_cast<float>(cum[i] - cum[j])) * iq[i] * ik[j] : 0.f;
      }
    }
    f32x4_t o[2];
#pragma unroll
    for (int ti = 0; ti < 2; ++ti) {
      f32x4_t ks = {0.f, 0.f, 0.f, 0.f};
      o[ti] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const f32x4_t kf = *reinterpret_cast<const f32x4_t*>(Ks + (16 * ti + i16) * LS + 16 * t + 4 * g);
        const f32x4_t qf = *reinterpret_cast<const f32x4_t*>(Qs + (16 * ti + i16) * LS + 16 * t + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          ks = mfma4(kf[r], s[t][r], ks);
          o[ti] = mfma4(qf[r], s[t][r], o[ti]);
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * ti + 4 * g + r;
        const float e = expf(static_cast<float>(cum[i]));
        u[ti][r] = beta[i] * (u[ti][r] - e * ik[i] * ks[r]);
        o[ti][r] *= e * iq[i];
      }
    }
    __syncthreads();
    f32x4_t rhs[2] = {u[0], u[1]};
#pragma unroll
    for (int ti = 0; ti < 2; ++ti) {
      u[ti] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int tj = 0; tj <= ti; ++tj) {
        const f32x4_t w = *reinterpret_cast<const f32x4_t*>(As + (16 * ti + i16) * kSq + 16 * tj + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) u[ti] = mfma4(w[r], rhs[tj][r], u[ti]);
      }
    }
#pragma unroll
    for (int ti = 0; ti < 2; ++ti)
#pragma unroll
      for (int tj = 0; tj <= ti; ++tj) {
        const f32x4_t w = *reinterpret_cast<const f32x4_t*>(Ps + (16 * ti + i16) * kSq + 16 * tj + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) o[ti] = mfma4(w[r], u[tj][r], o[ti]);
      }
#pragma unroll
    for (int ti = 0; ti < 2; ++ti)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * ti + 4 * g + r;
        if (live && i < len) st1(op + static_cast<int64_t>(c0 + i) * p.o_stride, o[ti][r]);
      }
    const double cn = cum[kQ - 1];
    const float fix = expf(static_cast<float>(cn));
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * tj + 4 * g + r;
        u[tj][r] *= expf(static_cast<float>(cn - cum[j])) * ik[j];
      }
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      s[t] *= fix;
#pragma unroll
      for (int tj = 0; tj < 2; ++tj)
#pragma unroll
        for (int r = 0; r < 4; ++r) s[t] = mfma4(Ks[(16 * tj + 4 * g + r) * LS + 16 * t + i16], u[tj][r], s[t]);
    }
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = 16 * t + 4 * g + r;
      if (live && n < p.K) S[static_cast<int64_t>(n) * p.V] = s[t][r];
    }
}

struct MemoryChunkParams {
  const void *q, *k, *v, *gi, *gf;
  int64_t stride;
  const float *bi, *bf;
  float *state, *norm;       // norm: [slots, heads, blocks, D + 1], one copy per 16 value columns (recurrent.hip)
  const int64_t* slots;
  const int64_t* positions;
  const int32_t *seg_start, *seg_len;
  void* o;
  int64_t o_stride;
  int heads, D, V, blocks, vec, col_waves;
  float cap, q_scale;
};

template <typename T, int NT>
__global__ __launch_bounds__(256, NT <= 8 ? 2 : 1) void memory_chunk_kernel(MemoryChunkParams p) {
  constexpr int NP = NT * 16, LS = NP + 4;
  __shared__ __attribute__((aligned(16))) float Ks[kQ * LS];
  __shared__ __attribute__((aligned(16))) float Qs[kQ * LS];
  __shared__ __attribute__((aligned(16))) float Gs[kQ * kSq];
  __shared__ __attribute__((aligned(16))) float ns[NP];
  // what the gates of a chunk make, formed a chunk ahead: a_j, g_i, e^{a_j-g_n}, e^{m0-g_i}, e^{-c_i-g_i}, and the m behind the chunk
  __shared__ double as[2][kQ], gs[2][kQ];
  __shared__ float add_w[2][kQ], keep_w[2][kQ], floor_w[2][kQ], m_next[2];
  __shared__ float inv[kQ];
  const int b = blockIdx.y, h = blockIdx.x;
  constexpr int waves = 4;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int block = blockIdx.z * p.col_waves, col = (block + wave) * 16 + i16;
  const bool live = wave < p.col_waves && col < p.V;           // waves without columns only help with the shared matrices
  const int64_t t0 = p.seg_start[b];
  const int total = p.seg_len[b];
  if (total <= 0) return;
  const int64_t pos0 = p.positions[t0], head = p.slots[b] * p.heads + h;
  float* S = p.state + head * p.D * p.V + col;
  float* norm = p.norm + (head * p.blocks + block) * (p.D + 1);
  f32x4_t s[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = 16 * t + 4 * g + r;
      s[t][r] = pos0 > 0 && live && n < p.D ? S[static_cast<int64_t>(n) * p.V] : 0.f;
    }
  if (threadIdx.x < NP) ns[threadIdx.x] = pos0 > 0 && static_cast<int>(threadIdx.x) < p.D ? norm[threadIdx.x] : 0.f;
  float m0 = pos0 > 0 ? norm[p.D] : 0.f;
  const float bi = p.bi[h], bf = p.bf[h];
  const T* qp = static_cast<const T*>(p.q) + t0 * p.stride + h * p.D;
  const T* kp = static_cast<const T*>(p.k) + t0 * p.stride + h * p.D;
  const T* vp = static_cast<const T*>(p.v) + t0 * p.stride + h * p.V + col;
  const T* ip = static_cast<const T*>(p.gi) + t0 * p.stride + h;
  const T* fp = static_cast<const T*>(p.gf) + t0 * p.stride + h;
  T* op = static_cast<T*>(p.o) + t0 * p.o_stride + h * p.V + col;

  RowTile<T, NP> qt, kt;
  T vr[2][4], ir = T{}, fr = T{};
  auto fetch = [&](int c0) __attribute__((always_inline)) {
    const int len = total - c0 < kQ ? total - c0 : kQ;
    const int64_t row = static_cast<int64_t>(c0) * p.stride;
    qt.fetch(qp + row, p.stride, len, p.D, p.vec);
    kt.fetch(kp + row, p.stride, len, p.D, p.vec);
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * tj + 4 * g + r;
        vr[tj][r] = live && j < len ? vp[row + j * p.stride] : T{};
      }
  };
  // the last wave, which has no part in the Gram tiles, fetches the gates two chunks ahead and scans them one chunk ahead
  auto fetch_gates = [&](int c0) __attribute__((always_inline)) {
    if (c0 + lane < total && lane < kQ) {
      ir = ip[(c0 + lane) * p.stride];
      fr = fp[(c0 + lane) * p.stride];
    }
  };
  auto scan_gates = [&](int c0, int to, float from) __attribute__((always_inline)) {
    const bool in = lane < kQ && c0 + lane < total;
    const float gi = p.cap * tanhf((ld1(&ir) + bi) / p.cap), gf = -softplus_f(-p.cap * tanhf((ld1(&fr) + bf) / p.cap));
    const double c = scan32(in ? static_cast<double>(gf) : 0.0, lane), start = from;
    const double a = in ? static_cast<double>(gi) - c : -INFINITY;
    double top = a > start ? a : start;
#pragma unroll
    for (int off = 1; off < kQ; off <<= 1) {
      const double u = __shfl_up(top, off, 64);
      if (lane >= off && u > top) top = u;
    }
    const double gn = __shfl(top, kQ - 1, 64);
    if (lane < kQ) {
      as[to][lane] = a;
      gs[to][lane] = top;
      add_w[to][lane] = expf(static_cast<float>(a - gn));
      keep_w[to][lane] = expf(static_cast<float>(start - top));
      floor_w[to][lane] = expf(static_cast<float>(-(c + top)));
      if (lane == kQ - 1) m_next[to] = static_cast<float>(c + top);      // (what a state of its own would hold)
    }
  };
  fetch(0);
  if (wave == waves - 1) {
    fetch_gates(0);
    scan_gates(0, 0, m0);
    fetch_gates(kQ);
  }
  for (int c0 = 0; c0 < total; c0 += kQ) {
    const int len = total - c0 < kQ ? total - c0 : kQ;
    qt.commit(Qs, LS);
    kt.commit(Ks, LS);
    const int at = (c0 / kQ) & 1;
    float x[2][4];
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) x[tj][r] = ld1(&vr[tj][r]);
    __syncthreads();
    if (c0 + kQ < total) fetch(c0 + kQ);
    for (int tile = wave; tile < 3; tile += waves) {
      const int ti = tile > 0, tj = tile > 1;
      const f32x4_t gm = gram_tile(Qs + 16 * ti * LS, Ks + 16 * tj * LS, NP, LS, i16, g);
      const int j = 16 * tj + i16;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * ti + 4 * g + r;
        Gs[i * kSq + j] = j <= i ? gm[r] * p.q_scale * expf(static_cast<float>(as[at][j] - gs[at][i])) : 0.f;
      }
    }
    if (wave == waves - 1 && c0 + kQ < total) {
      scan_gates(c0 + kQ, at ^ 1, m_next[at]);
      fetch_gates(c0 + 2 * kQ);
    }
    f32x4_t y[2];
#pragma unroll
    for (int ti = 0; ti < 2; ++ti) {
      y[ti] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const f32x4_t q = *reinterpret_cast<const f32x4_t*>(Qs + (16 * ti + i16) * LS + 16 * t + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) y[ti] = mfma4(q[r], s[t][r], y[ti]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) y[ti][r] *= p.q_scale * keep_w[at][16 * ti + 4 * g + r];
    }
    __syncthreads();
    {                                                  // denominators: eight lanes a token
      const int i = threadIdx.x >> 3, e = (threadIdx.x & 7) * 4;
      float d = 0.f;
      for (int c = e; c < NP; c += 32) {
        const f32x4_t q = *reinterpret_cast<const f32x4_t*>(Qs + i * LS + c), n = *reinterpret_cast<const f32x4_t*>(ns + c);
        d += q[0] * n[0] + q[1] * n[1] + q[2] * n[2] + q[3] * n[3];
      }
      d *= p.q_scale * keep_w[at][i];
      if (e < 16 || i >= 16) {                         // (the block above the diagonal is not formed)
        const f32x4_t w = *reinterpret_cast<const f32x4_t*>(Gs + i * kSq + e);
        d += w[0] + w[1] + w[2] + w[3];
      }
      d += __shfl_xor(d, 1, 64);
      d += __shfl_xor(d, 2, 64);
      d += __shfl_xor(d, 4, 64);
      if (e == 0) inv[i] = 1.0f / (fmaxf(fabsf(d), floor_w[at][i]) + 1e-6f);
    }
#pragma unroll
    for (int ti = 0; ti < 2; ++ti)
#pragma unroll
      for (int tj = 0; tj <= ti; ++tj) {
        const f32x4_t w = *reinterpret_cast<const f32x4_t*>(Gs + (16 * ti + i16) * kSq + 16 * tj + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r) y[ti] = mfma4(w[r], x[tj][r], y[ti]);
      }
    const float fix = keep_w[at][kQ - 1];
#pragma unroll
    for (int tj = 0; tj < 2; ++tj)
#pragma unroll
      for (int r = 0; r < 4; ++r) x[tj][r] *= add_w[at][16 * tj + 4 * g + r];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      s[t] *= fix;
#pragma unroll
      for (int tj = 0; tj < 2; ++tj)
#pragma unroll
        for (int r = 0; r < 4; ++r) s[t] = mfma4(Ks[(16 * tj + 4 * g + r) * LS + 16 * t + i16], x[tj][r], s[t]);
    }
    __syncthreads();
#pragma unroll
    for (int ti = 0; ti < 2; ++ti)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * ti + 4 * g + r;
        if (live && i < len) st1(op + static_cast<int64_t>(c0 + i) * p.o_stride, y[ti][r] * inv[i]);
      }
    if (threadIdx.x < NP) {
      float n = ns[threadIdx.x] * fix;
#pragma unroll 8
      for (int j = 0; j < kQ; ++j) n += Ks[j * LS + threadIdx.x] * add_w[at][j];      // (rows behind the last are zero)
      ns[threadIdx.x] = n;
    }
    m0 = m_next[at];
    __syncthreads();
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = 16 * t + 4 * g + r;
      if (live && n < p.D) S[static_cast<int64_t>(n) * p.V] = s[t][r];
    }
  for (int w = 0; w < p.col_waves && block + w < p.blocks; ++w) {
    if (static_cast<int>(threadIdx.x) < p.D) norm[w * (p.D + 1) + threadIdx.x] = ns[threadIdx.x];
    if (threadIdx.x == 0) norm[w * (p.D + 1) + p.D] = m0;
  }
}

// Columns per workgroup in waves of 16: up to 64, fewer while the launch would leave compute units empty.
int column_waves(int cols, int64_t segs_heads) {
  int w = (cols + 15) / 16;
  if (w > 4) w = 4;
  while (w > 1 && segs_heads * ((cols + 16 * w - 1) / (16 * w)) < 256) w /= 2;
  return w;
}

template <typename T>
void launch_mamba2_chunk(Mamba2ChunkParams p, int segs, hipStream_t st) {
  const int w = p.col_waves = column_waves(p.P, static_cast<int64_t>(segs) * p.heads);
  const dim3 grid(p.heads, segs, (p.P + 16 * w - 1) / (16 * w)), block(256);
  const int nt = (p.N + 15) / 16;
  if (nt <= 2) hipLaunchKernelGGL((mamba2_chunk_kernel<T, 2>), grid, block, 0, st, p);
  else if (nt <= 4) hipLaunchKernelGGL((mamba2_chunk_kernel<T, 4>), grid, block, 0, st, p);
  else if (nt <= 8) hipLaunchKernelGGL((mamba2_chunk_kernel<T, 8>), grid, block, 0, st, p);
  else hipLaunchKernelGGL((mamba2_chunk_kernel<T, 12>), grid, block, 0, st, p);
}

template <typename T>
void launch_delta_chunk(DeltaChunkParams p, int segs, hipStream_t st) {
  const int w = p.col_waves = column_waves(p.V, static_cast<int64_t>(segs) * p.heads);
  const dim3 grid(p.heads, segs, (p.V + 16 * w - 1) / (16 * w)), block(256);
  const int nt = (p.K + 15) / 16;
  if (nt <= 2) hipLaunchKernelGGL((delta_chunk_kernel<T, 2>), grid, block, 0, st, p);
  else if (nt <= 4) hipLaunchKernelGGL((delta_chunk_kernel<T, 4>), grid, block, 0, st, p);
  else if (nt <= 8) hipLaunchKernelGGL((delta_chunk_kernel<T, 8>), grid, block, 0, st, p);
  else hipLaunchKernelGGL((delta_chunk_kernel<T, 12>), grid, block, 0, st, p);
}

template <typename T>
void launch_memory_chunk(MemoryChunkParams p, int segs, hipStream_t st) {
  const int w = p.col_waves = column_waves(p.V, static_cast<int64_t>(segs) * p.heads);
  const dim3 grid(p.heads, segs, (p.V + 16 * w - 1) / (16 * w)), block(256);
  const int nt = (p.D + 15) / 16;
  if (nt <= 2) hipLaunchKernelGGL((memory_chunk_kernel<T, 2>), grid, block, 0, st, p);
  else if (nt <= 4) hipLaunchKernelGGL((memory_chunk_kernel<T, 4>), grid, block, 0, st, p);
  else if (nt <= 8) hipLaunchKernelGGL((memory_chunk_kernel<T, 8>), grid, block, 0, st, p);
  else hipLaunchKernelGGL((memory_chunk_kernel<T, 12>), grid, block, 0, st, p);
}

}  // namespace

extern "C" {

int sgl_amd_recurrent_chunk_max_state(void) { return 192; }

int sgl_amd_mamba2_chunk(int is_f32, const void* xbc, int64_t xbc_stride, const void* dt, int64_t dt_stride, const float* A_log,
                         const float* dt_bias, const float* D, float* state, const int64_t* slots, const int64_t* positions,
                         const int32_t* seg_start, const int32_t* seg_len, void* y, int64_t y_stride, int segments, int heads, int head_dim,
                         int state_dim, int groups, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(xbc && dt && A_log && dt_bias && D && state && slots && positions && seg_start && seg_len && y, "mamba2_chunk: null operand");
  SGL_CHECK_ARG(groups > 0 && heads > 0 && heads % groups == 0 && head_dim > 0 && state_dim > 0 && state_dim <= 192 && segments <= 65535,
                "mamba2_chunk: %d heads in %d groups, state %d (at most 192)", heads, groups, state_dim);
  if (segments <= 0) return 0;
  const size_t al = is_f32 ? 16 : 8;
  const int vec = state_dim % 4 == 0 && xbc_stride % 4 == 0 && (heads * head_dim) % 4 == 0 && aligned_to(xbc, al);
  Mamba2ChunkParams p{xbc, xbc_stride, dt, dt_stride, A_log, dt_bias, D, state, slots, positions, seg_start, seg_len, y, y_stride,
                      heads, head_dim, state_dim, groups, vec, 0};
  if (is_f32) launch_mamba2_chunk<float>(p, segments, as_stream(stream));
  else launch_mamba2_chunk<uint16_t>(p, segments, as_stream(stream));
  SGL_CHECK_LAUNCH("mamba2_chunk");
  return 0;
}

int sgl_amd_delta_chunk(int is_f32, const void* qkv, int64_t qkv_stride, const void* b, const void* a, int64_t ba_stride,
                        const float* A_log, const float* dt_bias, float* state, const int64_t* slots, const int64_t* positions,
                        const int32_t* seg_start, const int32_t* seg_len, void* o, int64_t o_stride, int segments, int heads, int kv_heads,
                        int key_dim, int value_dim, float q_scale, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(qkv && b && a && A_log && dt_bias && state && slots && positions && seg_start && seg_len && o, "delta_chunk: null operand");
  SGL_CHECK_ARG(kv_heads > 0 && heads > 0 && heads % kv_heads == 0 && value_dim > 0 && key_dim > 0 && key_dim <= 192 && segments <= 65535,
                "delta_chunk: %d value heads over %d key heads, key dim %d (at most 192)", heads, kv_heads, key_dim);
  if (segments <= 0) return 0;
  const size_t al = is_f32 ? 16 : 8;
  const int vec = key_dim % 4 == 0 && qkv_stride % 4 == 0 && aligned_to(qkv, al);
  DeltaChunkParams p{qkv, qkv_stride, b, a, ba_stride, A_log, dt_bias, state, slots, positions, seg_start, seg_len, o, o_stride,
                     heads, kv_heads, key_dim, value_dim, vec, 0, q_scale};
  if (is_f32) launch_delta_chunk<float>(p, segments, as_stream(stream));
  else launch_delta_chunk<uint16_t>(p, segments, as_stream(stream));
  SGL_CHECK_LAUNCH("delta_chunk");
  return 0;
}

int sgl_amd_memory_chunk(int is_f32, const void* q, const void* k, const void* v, const void* gate_i, const void* gate_f, int64_t stride,
                         const float* bias_i, const float* bias_f, float* state, float* norm, const int64_t* slots, const int64_t* positions,
                         const int32_t* seg_start, const int32_t* seg_len, void* o, int64_t o_stride, int segments, int heads, int key_dim,
                         int value_dim, float gate_cap, float q_scale, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(q && k && v && gate_i && gate_f && bias_i && bias_f && state && norm && slots && positions && seg_start && seg_len && o,
                "memory_chunk: null operand");
  SGL_CHECK_ARG(heads > 0 && value_dim > 0 && key_dim > 0 && key_dim <= 192 && segments <= 65535 && gate_cap > 0.f,
                "memory_chunk: %d heads of %d x %d (keys at most 192), gate cap %g", heads, key_dim, value_dim, gate_cap);
  if (segments <= 0) return 0;
  const size_t al = is_f32 ? 16 : 8;
  const int vec = key_dim % 4 == 0 && stride % 4 == 0 && aligned_to(q, al) && aligned_to(k, al);
  MemoryChunkParams p{q, k, v, gate_i, gate_f, stride, bias_i, bias_f, state, norm, slots, positions, seg_start, seg_len, o, o_stride,
                      heads, key_dim, value_dim, (value_dim + 15) / 16, vec, 0, gate_cap, q_scale};
  if (is_f32) launch_memory_chunk<float>(p, segments, as_stream(stream));
  else launch_memory_chunk<uint16_t>(p, segments, as_stream(stream));
  SGL_CHECK_LAUNCH("memory_chunk");
  return 0;
}

}  // extern "C"
