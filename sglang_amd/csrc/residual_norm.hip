// Row kernels around an fp32 residual stream, and the gated norms behind recurrent mixers.
//
//   residual_norm   one launch between two sublayers:  x <- source  (embedding row, x + LayerNorm(y), or y + vector),
//                   then optionally h = LayerNorm(x) for the next projection and copies of x in the activation type.
//                   The residual row lives in fp32 and is in registers for both norms.
//   residual_rms    the same step of pre-norm designs with RMS norms:  x <- embedding (+ position row), or x + up to two sublayer
//                   outputs (rows, split-K partials, or weighted expert rows), then a saved copy, then + rows + vector in front
//                   of a looped pass, then h = RMS norm(x).  Post-norm designs: x + mult * RMS norm(sum of the outputs), h = x or its norm.
//                   In decode batches h may leave blended with the row its request left one token ago (token shift)
//   soft_cap        cap * tanh(z / cap) on logits, fp32 out
//   gated_rmsnorm   RMS norm of equal column groups with a silu gate, the gate before the norm (Mamba-2) or behind it
//                   (gated delta rule), or with a sigmoid gate behind the norm (matrix memory).
//   gate_mul        act(a) * b for activation types / alignments outside silu_and_mul's bf16 form.
//   squared_relu    relu(a)^2, in place or not.
#include "elem_io.hpp"
#include "glu.hpp"
#include "sglang_amd.h"

using namespace sgl_amd;

namespace {

struct ResidualNormParams {
  int mode;                 // 0: x = table[ids] * scale   1: x += LN(y; w1, b1)   2: x = y + step
  const int64_t* ids;
  const void* table;        // [vocab, W]
  int64_t vocab;
  float scale;
  const void* y;            // [rows, W] activation type
  int64_t y_stride;
  const float* part;        // or the split-K partials of y, fp32 [splits, rows, W], summed in split order
  int splits;
  const void* part_bias;    // optional [W], activation type
  const float* step;        // [W]
  const float *w1, *b1;     // LayerNorm of y
  float* x;                 // [rows, W] fp32
  int64_t x_stride;
  const float *w2, *b2;     // LayerNorm of the new x -> h (h may be null)
  void* h;
  int64_t h_stride;
  void *copy0, *copy1;      // optional copies of the new x in the activation type
  int64_t copy_stride;
  int64_t rows;
  int width;
  float eps;
};

// Every thread owns kItems groups of VEC consecutive columns; the norm parameters of those columns stay in registers over
// the rows a workgroup walks (kHold), or are read where they are used (wide or unaligned rows).
template <typename T, int VEC, int kItems, bool kHold, bool kPart>
__global__ void residual_norm_kernel(ResidualNormParams p) {
  __shared__ float scratch[16];
  const int W = p.width;
  const float inv_w = 1.0f / static_cast<float>(W);
  constexpr int kKeep = kHold ? kItems : 1;
  float w1[kKeep][VEC], b1[kKeep][VEC], w2[kKeep][VEC], b2[kKeep][VEC];
#pragma unroll
  for (int i = 0; i < kKeep; ++i) {
    const int c = (i * blockDim.x + threadIdx.x) * VEC;
    if (kHold && c < W) {
      if (p.mode == 1) { ldv<VEC>(p.w1 + c, w1[i]); ldv<VEC>(p.b1 + c, b1[i]); }
      if (p.mode == 2) ldv<VEC>(p.step + c, b1[i]);
      if (p.h) { ldv<VEC>(p.w2 + c, w2[i]); ldv<VEC>(p.b2 + c, b2[i]); }
    }
  }
  for (int64_t row = blockIdx.x; row < p.rows; row += gridDim.x) {
    float v[kItems][VEC];
    float* xr = p.x + row * p.x_stride;
    if (p.mode == 0) {
      int64_t id = p.ids[row];
      if (id < 0 || id >= p.vocab) id = 0;
      const T* tr = static_cast<const T*>(p.table) + id * W;
#pragma unroll
      for (int i = 0; i < kItems; ++i) {
        const int c = (i * blockDim.x + threadIdx.x) * VEC;
        if (c < W) {
          ldv<VEC>(tr + c, v[i]);
#pragma unroll
          for (int j = 0; j < VEC; ++j) v[i][j] *= p.scale;
        }
      }
    } else {
      const T* yr = static_cast<const T*>(p.y) + row * p.y_stride;
      float old[kKeep][VEC];
#pragma unroll
      for (int i = 0; i < kItems; ++i) {
        const int c = (i * blockDim.x + threadIdx.x) * VEC;
        if (c < W) {
          if constexpr (kPart) {
            const float* src = p.part + row * W + c;
            ldv<VEC>(src, v[i]);
            for (int s = 1; s < p.splits; s += 4) {            // four loads in flight, clamped to the last split
              float u[4][VEC];
#pragma unroll
              for (int q = 0; q < 4; ++q) ldv<VEC>(src + static_cast<int64_t>(s + q < p.splits ? s + q : p.splits - 1) * p.rows * W, u[q]);
#pragma unroll
              for (int q = 0; q < 4; ++q)
                if (s + q < p.splits) {
#pragma unroll
                  for (int j = 0; j < VEC; ++j) v[i][j] += u[q][j];
                }
            }
            if (p.part_bias) {
              float bv[VEC];
              ldv<VEC>(static_cast<const T*>(p.part_bias) + c, bv);
#pragma unroll
              for (int j = 0; j < VEC; ++j) v[i][j] += bv[j];
            }
          } else {
            ldv<VEC>(yr + c, v[i]);
          }
          if (kHold && p.mode == 1) ldv<VEC>(xr + c, old[kHold ? i : 0]);
        }
      }
      if (p.mode == 2) {
#pragma unroll
        for (int i = 0; i < kItems; ++i) {
          const int c = (i * blockDim.x + threadIdx.x) * VEC;
          if (c < W) {
            if (!kHold) ldv<VEC>(p.step + c, b1[0]);
#pragma unroll
            for (int j = 0; j < VEC; ++j) v[i][j] += b1[kHold ? i : 0][j];
          }
        }
      } else {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < kItems; ++i)
          if ((i * blockDim.x + threadIdx.x) * VEC < W) {
#pragma unroll
            for (int j = 0; j < VEC; ++j) s += v[i][j];
          }
        const float mean = block_sum(s, scratch) * inv_w;
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < kItems; ++i)
          if ((i * blockDim.x + threadIdx.x) * VEC < W) {
#pragma unroll
            for (int j = 0; j < VEC; ++j) { const float d = v[i][j] - mean; ss += d * d; }
          }
        const float rs = 1.0f / sqrtf(block_sum(ss, scratch) * inv_w + p.eps);
#pragma unroll
        for (int i = 0; i < kItems; ++i)
          if (const int c = (i * blockDim.x + threadIdx.x) * VEC; c < W) {
            if (!kHold) { ldv<VEC>(p.w1 + c, w1[0]); ldv<VEC>(p.b1 + c, b1[0]); ldv<VEC>(xr + c, old[0]); }
#pragma unroll
            for (int j = 0; j < VEC; ++j)
              v[i][j] = old[kHold ? i : 0][j] + ((v[i][j] - mean) * rs * w1[kHold ? i : 0][j] + b1[kHold ? i : 0][j]);
          }
      }
    }
#pragma unroll
    for (int i = 0; i < kItems; ++i) {
      const int c = (i * blockDim.x + threadIdx.x) * VEC;
      if (c < W) {
        stv<VEC>(xr + c, v[i]);
        if (p.copy0) stv<VEC>(static_cast<T*>(p.copy0) + row * p.copy_stride + c, v[i]);
        if (p.copy1) stv<VEC>(static_cast<T*>(p.copy1) + row * p.copy_stride + c, v[i]);
      }
    }
    if (p.h) {
      float s = 0.f;
#pragma unroll
      for (int i = 0; i < kItems; ++i)
        if ((i * blockDim.x + threadIdx.x) * VEC < W) {
#pragma unroll
          for (int j = 0; j < VEC; ++j) s += v[i][j];
        }
      const float mean = block_sum(s, scratch) * inv_w;
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < kItems; ++i)
        if ((i * blockDim.x + threadIdx.x) * VEC < W) {
#pragma unroll
          for (int j = 0; j < VEC; ++j) { const float d = v[i][j] - mean; ss += d * d; }
        }
      const float rs = 1.0f / sqrtf(block_sum(ss, scratch) * inv_w + p.eps);
      T* hr = static_cast<T*>(p.h) + row * p.h_stride;
#pragma unroll
      for (int i = 0; i < kItems; ++i) {
        const int c = (i * blockDim.x + threadIdx.x) * VEC;
        if (c < W) {
          float o[VEC];
          if (!kHold) { ldv<VEC>(p.w2 + c, w2[0]); ldv<VEC>(p.b2 + c, b2[0]); }
#pragma unroll
          for (int j = 0; j < VEC; ++j) o[j] = (v[i][j] - mean) * rs * w2[kHold ? i : 0][j] + b2[kHold ? i : 0][j];
          stv<VEC>(hr + c, o);
        }
      }
    }
  }
}

template <typename T, int VEC, int kItems, bool kHold>
void launch_residual_norm(const ResidualNormParams& p, hipStream_t st) {
  const int per = VEC * kItems;
  int threads = ((p.width + per - 1) / per + 63) / 64 * 64;
  if (threads > 1024) threads = 1024;
  const int64_t cap = 256 * (2048 / threads);
  const dim3 grid(static_cast<unsigned>(p.rows < cap ? p.rows : cap));
  if (p.part) hipLaunchKernelGGL((residual_norm_kernel<T, VEC, kItems, kHold, true>), grid, dim3(threads), 0, st, p);
  else hipLaunchKernelGGL((residual_norm_kernel<T, VEC, kItems, kHold, false>), grid, dim3(threads), 0, st, p);
}

template <typename T>
void launch_residual_norm_t(const ResidualNormParams& p, bool vec, hipStream_t st) {
  if (vec && p.width <= 4 * 1024) launch_residual_norm<T, 4, 1, true>(p, st);
  else if (vec && p.width <= 8 * 1024) launch_residual_norm<T, 4, 2, true>(p, st);
  else if (vec) launch_residual_norm<T, 4, 4, false>(p, st);
  else launch_residual_norm<T, 1, 16, false>(p, st);
}

// ---------------------------------------------------------------------------------------------------------------
// One addend of a residual row: the sum over i < n of weight[row, i] * data[row * row_stride + i * item_stride + column].  An item whose
// id is negative is the row of `alt` instead (an expert that hands on its input).
struct RowSource {
  const void* data;
  int f32;                  // element type: fp32, else the activation type
  int n;
  int64_t row_stride, item_stride;
  const float* weight;      // element (row, i) at row * w_row + i * w_item, or null: all ones
  int64_t w_row, w_item;
  const int32_t* ids;       // [rows, n], or null
  const void* alt;          // activation type
  int64_t alt_stride;
};

struct ResidualRmsParams {
  const int64_t* ids;       // embedding form: x = table[ids] * scale + pos_table[positions]
  const void* table;
  int64_t vocab;
  float scale;
  const int64_t* positions;
  const void* pos_table;    // may be null
  int64_t max_pos;
  RowSource a, b;           // otherwise x = x + a + b (either may be absent)
  float* x;                 // [rows, W] fp32
  int64_t x_stride;
  float* save;              // optional fp32 copy of x as it is here
  const float* extra;       // optional fp32 rows, added behind the copy (the stride of `save` / `extra` is W)
  const float* step;        // optional [W], added last
  const float* bias;        // optional [W], part of the addends' sum
  const float* post;        // optional [W]: x = x + mult * (RMS norm(a + b) * post)
  float mult;
  const float* w;           // [W]; null: h is the new x itself
  void* h;                  // RMS norm of the new x (may be null)
  int64_t h_stride;
  const float* shift;       // optional [W]: h = norm + (the row's norm one token ago - norm) * shift; the norm goes to the state
  void* shift_state;        // [slots, W] activation type
  const int64_t *shift_slots, *shift_pos;      // [rows]; position 0: nothing in front
  int64_t rows;
  int width;
  float eps;
};

// kMore: items may be another row
template <typename T, bool kMore>
__device__ __forceinline__ const T* source_item(const RowSource& s, int64_t row, int i) {
  if (kMore && s.ids && s.ids[row * s.n + i] < 0) return static_cast<const T*>(s.alt) + row * s.alt_stride;
  return static_cast<const T*>(s.data) + row * s.row_stride + i * s.item_stride;
}

template <typename T, int VEC, bool kMore>
__device__ __forceinline__ void add_source(const RowSource& s, int64_t row, int c, float (&v)[VEC]) {
  const float* wr = s.weight ? s.weight + row * s.w_row : nullptr;
  for (int i = 0; i < s.n; i += 4) {                  // four loads in flight, clamped to the last item
    float u[4][VEC];
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int item = i + q < s.n ? i + q : s.n - 1;
      if (s.f32) ldv<VEC>(source_item<float, kMore>(s, row, item) + c, u[q]);
      else ldv<VEC>(source_item<T, kMore>(s, row, item) + c, u[q]);
    }
#pragma unroll
    for (int q = 0; q < 4; ++q)
      if (i + q < s.n) {
        const float f = wr ? wr[(i + q) * s.w_item] : 1.0f;
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += f * u[q][j];
      }
  }
}

// The same over all the columns of a thread: one item at a time, its pieces in flight together.
template <typename T, int VEC, int kItems, bool kMore>
__device__ __forceinline__ void add_source_row(const RowSource& s, int64_t row, int lane, int tpr, int W, float (&v)[kItems][VEC]) {
  constexpr int kAhead = kItems <= 4 ? 2 : 1;
#pragma unroll kAhead
  for (int q = 0; q < s.n; ++q) {
    const float f = s.weight ? s.weight[row * s.w_row + q * s.w_item] : 1.0f;
    const void* item = s.f32 ? static_cast<const void*>(source_item<float, kMore>(s, row, q)) : source_item<T, kMore>(s, row, q);
    float u[kItems][VEC];
#pragma unroll
    for (int i = 0; i < kItems; ++i) {
      int c = (i * tpr + lane) * VEC;
      if (c >= W) c = 0;
      if (s.f32) ldv<VEC>(static_cast<const float*>(item) + c, u[i]);
      else ldv<VEC>(static_cast<const T*>(item) + c, u[i]);
    }
#pragma unroll
    for (int i = 0; i < kItems; ++i)
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[i][j] += f * u[i][j];
  }
}

// kWaveRow: a wave owns a row (many rows: no barrier), else a workgroup does (decode batches: shortest path to one row).  kMore: with
// items that are another row, a bias, or a shift.
template <typename T, int VEC, int kItems, bool kWaveRow, bool kMore>
__global__ __launch_bounds__(kWaveRow ? 256 : 1024) void residual_rms_kernel(ResidualRmsParams p) {
  __shared__ float scratch[16];
  const int tpr = kWaveRow ? 64 : static_cast<int>(blockDim.x);
  const int lane = kWaveRow ? threadIdx.x & 63 : threadIdx.x;
  const int64_t row = kWaveRow ? static_cast<int64_t>(blockIdx.x) * (blockDim.x >> 6) + (threadIdx.x >> 6) : blockIdx.x;
  if (row >= p.rows) return;                          // (whole waves, and whole workgroups where barriers follow)
  const int W = p.width;
  float v[kItems][VEC];
  float* xr = p.x + row * p.x_stride;
  if (p.ids) {
    int64_t id = p.ids[row];
    if (id < 0 || id >= p.vocab) id = 0;
    const T* tr = static_cast<const T*>(p.table) + id * W;
    const T* pr = nullptr;
    if (p.pos_table) {
      int64_t pos = p.positions[row];
      if (pos < 0 || pos >= p.max_pos) pos = p.max_pos - 1;      // (the host admits no such position)
      pr = static_cast<const T*>(p.pos_table) + pos * W;
    }
#pragma unroll
    for (int i = 0; i < kItems; ++i) {
      const int c = (i * tpr + lane) * VEC;
      if (c < W) {
        ldv<VEC>(tr + c, v[i]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[i][j] *= p.scale;
        if (pr) {
          float u[VEC];
          ldv<VEC>(pr + c, u);
#pragma unroll
          for (int j = 0; j < VEC; ++j) v[i][j] += u[j];
        }
      }
    }
  } else {
#pragma unroll
    for (int i = 0; i < kItems; ++i) {
      const int c = (i * tpr + lane) * VEC;
      if (p.post) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[i][j] = 0.f;
      } else if (c < W) {
        ldv<VEC>(xr + c, v[i]);
      }
    }
    if constexpr (kItems == 1) {
      if (lane * VEC < W) {
        if (p.a.data) add_source<T, VEC, kMore>(p.a, row, lane * VEC, v[0]);
        if (p.b.data) add_source<T, VEC, kMore>(p.b, row, lane * VEC, v[0]);
      }
    } else {
      if (p.a.data) add_source_row<T, VEC, kItems, kMore>(p.a, row, lane, tpr, W, v);
      if (p.b.data) add_source_row<T, VEC, kItems, kMore>(p.b, row, lane, tpr, W, v);
    }
    if (kMore && p.bias) {
#pragma unroll
      for (int i = 0; i < kItems; ++i) {
        const int c = (i * tpr + lane) * VEC;
        if (c < W) {
          float u[VEC];
          ldv<VEC>(p.bias + c, u);
#pragma unroll
          for (int j = 0; j < VEC; ++j) v[i][j] += u[j];
        }
      }
    }
    if (p.post) {
      float sq = 0.f;
#pragma unroll
      for (int i = 0; i < kItems; ++i)
        if ((i * tpr + lane) * VEC < W) {
#pragma unroll
          for (int j = 0; j < VEC; ++j) sq += v[i][j] * v[i][j];
        }
      sq = kWaveRow ? wave_sum(sq) : block_sum(sq, scratch);
      const float f = p.mult / sqrtf(sq / static_cast<float>(W) + p.eps);
#pragma unroll
      for (int i = 0; i < kItems; ++i) {
        const int c = (i * tpr + lane) * VEC;
        if (c < W) {
          float wv[VEC], old[VEC];
          ldv<VEC>(p.post + c, wv);
          ldv<VEC>(xr + c, old);
#pragma unroll
          for (int j = 0; j < VEC; ++j) v[i][j] = old[j] + v[i][j] * f * wv[j];
        }
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < kItems; ++i) {
    const int c = (i * tpr + lane) * VEC;
    if (c < W) {
      if (p.save) stv<VEC>(p.save + row * W + c, v[i]);
      float u[VEC];
      if (p.extra) {
        ldv<VEC>(p.extra + row * W + c, u);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[i][j] += u[j];
      }
      if (p.step) {
        ldv<VEC>(p.step + c, u);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[i][j] += u[j];
      }
      stv<VEC>(xr + c, v[i]);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss += v[i][j] * v[i][j];
    }
  }
  if (!p.h) return;
  T* hr = static_cast<T*>(p.h) + row * p.h_stride;
  if (!p.w) {
#pragma unroll
    for (int i = 0; i < kItems; ++i) {
      const int c = (i * tpr + lane) * VEC;
      if (c < W) stv<VEC>(hr + c, v[i]);
    }
    return;
  }
  ss = kWaveRow ? wave_sum(ss) : block_sum(ss, scratch);
  const float rs = 1.0f / sqrtf(ss / static_cast<float>(W) + p.eps);
  T* left = kMore && p.shift ? static_cast<T*>(p.shift_state) + p.shift_slots[row] * W : nullptr;
  const bool fresh = kMore && p.shift && p.shift_pos[row] <= 0;
#pragma unroll
  for (int i = 0; i < kItems; ++i) {
    const int c = (i * tpr + lane) * VEC;
    if (c < W) {
      float wv[VEC], o[VEC];
      ldv<VEC>(p.w + c, wv);
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = v[i][j] * rs * wv[j];
      if (kMore && p.shift) {
        float front[VEC], mu[VEC];
        ldv<VEC>(left + c, front);
        ldv<VEC>(p.shift + c, mu);
        stv<VEC>(left + c, o);
#pragma unroll
        for (int j = 0; j < VEC; ++j) o[j] += ((fresh ? 0.f : front[j]) - o[j]) * mu[j];
      }
      stv<VEC>(hr + c, o);
    }
  }
}

template <typename T, bool kMore>
void launch_residual_rms(const ResidualRmsParams& p, bool vec, bool vec8, hipStream_t st) {
  const unsigned by4 = static_cast<unsigned>((p.rows + 3) / 4), one = static_cast<unsigned>(p.rows);
  const int W = p.width;
  if (vec8 && p.rows >= 1024 && W <= 1024) hipLaunchKernelGGL((residual_rms_kernel<T, 8, 2, true, kMore>), dim3(by4), dim3(256), 0, st, p);
  else if (vec8 && p.rows >= 1024 && W <= 2048) hipLaunchKernelGGL((residual_rms_kernel<T, 8, 4, true, kMore>), dim3(by4), dim3(256), 0, st, p);
  else if (vec8 && p.rows >= 1024 && W <= 4096) hipLaunchKernelGGL((residual_rms_kernel<T, 8, 8, true, kMore>), dim3(by4), dim3(256), 0, st, p);
  else if (vec && W <= 4096) hipLaunchKernelGGL((residual_rms_kernel<T, 4, 1, false, kMore>), dim3(one), dim3((W / 4 + 63) / 64 * 64), 0, st, p);
  else if (vec) hipLaunchKernelGGL((residual_rms_kernel<T, 4, 4, false, kMore>), dim3(one), dim3(1024), 0, st, p);
  else hipLaunchKernelGGL((residual_rms_kernel<T, 1, 16, false, kMore>), dim3(one), dim3(W >= 1024 ? 1024 : (W + 63) / 64 * 64), 0, st, p);
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void soft_cap_kernel(const T* __restrict__ z, int64_t z_stride, int n, int64_t item_stride, float* __restrict__ out,
                                                       int cols, float cap, float inv_cap) {
  const int64_t row = blockIdx.y;
  const int c = (blockIdx.x * 256 + threadIdx.x) * VEC;
  if (c >= cols) return;
  float v[VEC];
  ldv<VEC>(z + row * z_stride + c, v);
  for (int i = 1; i < n; ++i) {
    float u[VEC];
    ldv<VEC>(z + i * item_stride + row * z_stride + c, u);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] += u[j];
  }
#pragma unroll
  for (int j = 0; j < VEC; ++j) v[j] = cap * tanhf(v[j] * inv_cap);
  stv<VEC>(out + row * cols + c, v);
}

template <typename T>
void launch_soft_cap(const void* z, int64_t z_stride, int n, int64_t item_stride, float* out, int64_t rows, int cols, float cap, hipStream_t st) {
  const bool vec = cols % 4 == 0 && z_stride % 4 == 0 && item_stride % 4 == 0 && aligned_to(z, sizeof(T) * 4) && aligned_to(out, 16);
  const int per = vec ? 1024 : 256;
  const dim3 grid((cols + per - 1) / per, static_cast<unsigned>(rows));
  if (vec) hipLaunchKernelGGL((soft_cap_kernel<T, 4>), grid, dim3(256), 0, st, static_cast<const T*>(z), z_stride, n, item_stride, out, cols, cap, 1.0f / cap);
  else hipLaunchKernelGGL((soft_cap_kernel<T, 1>), grid, dim3(256), 0, st, static_cast<const T*>(z), z_stride, n, item_stride, out, cols, cap, 1.0f / cap);
}

// ---------------------------------------------------------------------------------------------------------------
struct GatedNormParams {
  const void* y;       // [rows, groups * size]
  int64_t y_stride;
  const void* gate;    // same shape
  int64_t gate_stride;
  const float* w;      // [groups * size], or [size] shared by the groups
  void* out;
  int64_t out_stride;
  int64_t rows;
  int groups, size, gate_first, shared_w, gate_sigmoid;
  float eps;
};

// TPG threads share one (row, group); up to a wave, a 256-thread workgroup carries 256 / TPG of them.
template <typename T, int VEC, int TPG, int kItems>
__global__ void gated_rmsnorm_kernel(GatedNormParams p) {
  __shared__ float scratch[16];
  const int lane = threadIdx.x % TPG;
  const int64_t item = static_cast<int64_t>(blockIdx.x) * (blockDim.x / TPG) + threadIdx.x / TPG;
  const bool live = item < p.rows * p.groups;
  const int64_t row = live ? item / p.groups : 0;
  const int g = live ? static_cast<int>(item - row * p.groups) : 0;
  const T* yr = static_cast<const T*>(p.y) + row * p.y_stride + static_cast<int64_t>(g) * p.size;
  const T* gr = static_cast<const T*>(p.gate) + row * p.gate_stride + static_cast<int64_t>(g) * p.size;
  const float* wr = p.w + (p.shared_w ? 0 : static_cast<int64_t>(g) * p.size);
  T* orow = static_cast<T*>(p.out) + row * p.out_stride + static_cast<int64_t>(g) * p.size;
  float v[kItems][VEC], gt[kItems][VEC];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < kItems; ++i) {
    const int c = (i * TPG + lane) * VEC;
    if (live && c < p.size) {
      ldv<VEC>(yr + c, v[i]);
      ldv<VEC>(gr + c, gt[i]);
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        gt[i][j] = p.gate_sigmoid ? sigmoid_f(gt[i][j]) : silu_f(gt[i][j]);
        if (p.gate_first) v[i][j] *= gt[i][j];
        ss += v[i][j] * v[i][j];
      }
    }
  }
  if constexpr (TPG <= 64) {
#pragma unroll
    for (int off = TPG / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
  } else {
    ss = block_sum(ss, scratch);
  }
  const float rs = 1.0f / sqrtf(ss / static_cast<float>(p.size) + p.eps);
#pragma unroll
  for (int i = 0; i < kItems; ++i) {
    const int c = (i * TPG + lane) * VEC;
    if (live && c < p.size) {
      float wv[VEC], o[VEC];
      ldv<VEC>(wr + c, wv);
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        o[j] = v[i][j] * rs * wv[j];
        if (!p.gate_first) o[j] *= gt[i][j];
      }
      stv<VEC>(orow + c, o);
    }
  }
}

template <typename T, int VEC>
void launch_gated(const GatedNormParams& p, hipStream_t st) {
  const int64_t items = p.rows * p.groups;
  if (p.size <= 16 * VEC)
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, VEC, 16, 1>), dim3((items + 15) / 16), dim3(256), 0, st, p);
  else if (p.size <= 32 * VEC)
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, VEC, 32, 1>), dim3((items + 7) / 8), dim3(256), 0, st, p);
  else if (p.size <= 64 * VEC)
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, VEC, 64, 1>), dim3((items + 3) / 4), dim3(256), 0, st, p);
  else if (p.size <= 64 * VEC * 4)
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, VEC, 64, 4>), dim3((items + 3) / 4), dim3(256), 0, st, p);
  else if (p.size <= 256 * VEC * 4)
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, VEC, 256, 4>), dim3(items), dim3(256), 0, st, p);
  else
    hipLaunchKernelGGL((gated_rmsnorm_kernel<T, VEC, 1024, VEC == 4 ? 4 : 16>), dim3(items), dim3(1024), 0, st, p);
}

// ---------------------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void gate_mul_kernel(const T* __restrict__ a, const T* __restrict__ b, T* __restrict__ out, int d,
                                                       int64_t in_stride, int64_t out_stride, GluParams act) {
  const int64_t row = blockIdx.y;
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c < d) st1(out + row * out_stride + c, glu<false>(act, ld1(a + row * in_stride + c), ld1(b + row * in_stride + c)));
}

// Two vectors a thread.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void squared_relu_kernel(const T* a, T* out, int d, int64_t in_stride, int64_t out_stride) {
  const int64_t row = blockIdx.y;
  const int c0 = (blockIdx.x * 512 + threadIdx.x) * VEC;
  float v[2][VEC];
#pragma unroll
  for (int i = 0; i < 2; ++i)
    if (const int c = c0 + i * 256 * VEC; c < d) ldv<VEC>(a + row * in_stride + c, v[i]);
#pragma unroll
  for (int i = 0; i < 2; ++i)
    if (const int c = c0 + i * 256 * VEC; c < d) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[i][j] = squared_relu(v[i][j]);
      stv<VEC>(out + row * out_stride + c, v[i]);
    }
}

template <typename T>
void launch_squared_relu(const void* a, void* out, int64_t rows, int d, int64_t in_stride, int64_t out_stride, hipStream_t st) {
  const bool vec = d % 8 == 0 && in_stride % 8 == 0 && out_stride % 8 == 0 && aligned_to(a, 16) && aligned_to(out, 16);
  const int per = 512 * (vec ? 8 : 1);
  for (int64_t r = 0; r < rows; r += 65535) {
    const dim3 grid((d + per - 1) / per, static_cast<unsigned>(rows - r < 65535 ? rows - r : 65535));
    const T* ap = static_cast<const T*>(a) + r * in_stride;
    T* op = static_cast<T*>(out) + r * out_stride;
    if (vec) hipLaunchKernelGGL((squared_relu_kernel<T, 8>), grid, dim3(256), 0, st, ap, op, d, in_stride, out_stride);
    else hipLaunchKernelGGL((squared_relu_kernel<T, 1>), grid, dim3(256), 0, st, ap, op, d, in_stride, out_stride);
  }
}

}  // namespace

extern "C" {

int sgl_amd_residual_norm(int is_f32, int mode, const int64_t* ids, const void* table, int64_t vocab, float scale, const void* y,
                          int64_t y_stride, const float* partials, int splits, const void* partials_bias, const float* step, const float* w1, const float* b1, float* x, int64_t x_stride,
                          const float* w2, const float* b2, void* h, int64_t h_stride, void* copy0, void* copy1, int64_t copy_stride,
                          int64_t rows, int width, float eps, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(width > 0 && width <= 16384, "residual_norm: width %d outside 1..16384", width);
  SGL_CHECK_ARG(x && (mode == 0 ? (ids && table && vocab > 0) : mode == 1 ? ((y || partials) && w1 && b1) : (mode == 2 && (y || partials) && step)),
                "residual_norm: missing operand for mode %d", mode);
  SGL_CHECK_ARG(!h || (w2 && b2), "residual_norm: h needs its norm's parameters");
  SGL_CHECK_ARG(!partials || splits >= 1, "residual_norm: %d splits", splits);
  if (rows <= 0) return 0;
  ResidualNormParams p{mode, ids, table, vocab, scale, y, y_stride, partials, splits, partials_bias, step, w1, b1, x, x_stride, w2, b2, h, h_stride,
                       copy0, copy1, copy_stride, rows, width, eps};
  const size_t a = is_f32 ? 16 : 8;
  const bool vec = width % 4 == 0 && y_stride % 4 == 0 && x_stride % 4 == 0 && h_stride % 4 == 0 && copy_stride % 4 == 0 &&
                   aligned_to(table, a) && aligned_to(y, a) && aligned_to(partials, 16) && aligned_to(partials_bias, a) && aligned_to(h, a) && aligned_to(copy0, a) && aligned_to(copy1, a) &&
                   aligned_to(x, 16) && aligned_to(w1, 16) && aligned_to(b1, 16) && aligned_to(w2, 16) && aligned_to(b2, 16) &&
                   aligned_to(step, 16);
  if (is_f32) launch_residual_norm_t<float>(p, vec, as_stream(stream));
  else launch_residual_norm_t<uint16_t>(p, vec, as_stream(stream));
  SGL_CHECK_LAUNCH("residual_norm");
  return 0;
}

int sgl_amd_residual_rms(int is_f32, const int64_t* ids, const void* table, int64_t vocab, float scale, const int64_t* positions,
                         const void* pos_table, int64_t max_positions, const void* a, int a_f32, int a_items, int64_t a_row_stride,
                         int64_t a_item_stride, const float* a_weight, const void* b, int b_f32, int b_items, int64_t b_row_stride,
                         int64_t b_item_stride, const float* b_weight, float* x, int64_t x_stride, float* save, const float* extra,
                         const float* step, const float* post, float mult, const float* weight, void* h, int64_t h_stride, int64_t rows, int width,
                         float eps, int64_t a_weight_row, int64_t a_weight_item, const int32_t* a_ids, const void* a_alt, int64_t a_alt_stride,
                         int64_t b_weight_row, int64_t b_weight_item, const float* bias, const float* shift, void* shift_state,
                         const int64_t* shift_slots, const int64_t* shift_positions, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(width > 0 && width <= 16384, "residual_rms: width %d outside 1..16384", width);
  SGL_CHECK_ARG(x && (!ids || (table && vocab > 0 && !a && !b)) && (!pos_table || (ids && positions && max_positions > 0)),
                "residual_rms: missing operand, or an embedding beside sublayer outputs");
  SGL_CHECK_ARG((!a || a_items >= 1) && (!b || b_items >= 1) && (!post || a), "residual_rms: empty source, or a norm behind none");
  SGL_CHECK_ARG(!a_ids || (a && a_alt && (is_f32 || !a_f32)), "residual_rms: items that are another row need it, in the activation type");
  SGL_CHECK_ARG(!shift || (shift_state && shift_slots && shift_positions && weight && h), "residual_rms: a shift needs its state, slots, positions and norm");
  SGL_CHECK_ARG(rows <= 0x7fffffffLL, "residual_rms: too many rows");
  if (rows <= 0) return 0;
  ResidualRmsParams p{ids, table, vocab, scale, positions, pos_table, max_positions, {a, is_f32 || a_f32, a_items, a_row_stride, a_item_stride, a_weight, a_weight_row, a_weight_item, a_ids, a_alt, a_alt_stride},
                      {b, is_f32 || b_f32, b_items, b_row_stride, b_item_stride, b_weight, b_weight_row, b_weight_item, nullptr, nullptr, 0}, x, x_stride, save, extra,
                      step, bias, post, mult, weight, h, h_stride, shift, shift_state, shift_slots, shift_positions, rows, width, eps};
  const size_t al = is_f32 ? 16 : 8;
  const bool vec = width % 4 == 0 && x_stride % 4 == 0 && h_stride % 4 == 0 && a_row_stride % 4 == 0 && a_item_stride % 4 == 0 &&
                   b_row_stride % 4 == 0 && b_item_stride % 4 == 0 && aligned_to(table, al) && aligned_to(pos_table, al) &&
                   aligned_to(a, p.a.f32 ? 16 : 8) && aligned_to(b, p.b.f32 ? 16 : 8) && aligned_to(h, al) && aligned_to(x, 16) &&
                   aligned_to(save, 16) && aligned_to(extra, 16) && aligned_to(step, 16) && aligned_to(post, 16) && aligned_to(weight, 16) &&
                   aligned_to(bias, 16) && aligned_to(shift, 16) && aligned_to(shift_state, al) && a_alt_stride % 4 == 0 && aligned_to(a_alt, al);
  const bool vec8 = vec && width % 8 == 0 && h_stride % 8 == 0 && a_row_stride % 8 == 0 && a_item_stride % 8 == 0 && b_row_stride % 8 == 0 &&
                    b_item_stride % 8 == 0 && aligned_to(table, 16) && aligned_to(pos_table, 16) && aligned_to(a, 16) && aligned_to(b, 16) && aligned_to(h, 16) &&
                    a_alt_stride % 8 == 0 && aligned_to(a_alt, 16) && aligned_to(shift_state, 16);
  const bool more = a_ids || bias || shift;
  if (is_f32) more ? launch_residual_rms<float, true>(p, vec, vec8, as_stream(stream)) : launch_residual_rms<float, false>(p, vec, vec8, as_stream(stream));
  else more ? launch_residual_rms<uint16_t, true>(p, vec, vec8, as_stream(stream)) : launch_residual_rms<uint16_t, false>(p, vec, vec8, as_stream(stream));
  SGL_CHECK_LAUNCH("residual_rms");
  return 0;
}

int sgl_amd_soft_cap(int is_f32, const void* z, int64_t z_row_stride, int items, int64_t item_stride, float* out, int64_t rows, int cols,
                     float cap, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(z && out && cols > 0 && items >= 1 && cap > 0.f && rows <= 65535, "soft_cap: %d columns, %d items, cap %g", cols, items, cap);
  if (rows <= 0) return 0;
  if (is_f32) launch_soft_cap<float>(z, z_row_stride, items, item_stride, out, rows, cols, cap, as_stream(stream));
  else launch_soft_cap<uint16_t>(z, z_row_stride, items, item_stride, out, rows, cols, cap, as_stream(stream));
  SGL_CHECK_LAUNCH("soft_cap");
  return 0;
}

int sgl_amd_gated_rmsnorm(int is_f32, const void* y, int64_t y_stride, const void* gate, int64_t gate_stride, const float* weight,
                          void* out, int64_t out_stride, int64_t rows, int groups, int group_size, int gate_first, int shared_weight,
                          int gate_sigmoid, float eps, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(y && gate && weight && out && groups > 0 && group_size > 0 && group_size <= 16384,
                "gated_rmsnorm: %d groups of %d", groups, group_size);
  if (rows <= 0) return 0;
  GatedNormParams p{y, y_stride, gate, gate_stride, weight, out, out_stride, rows, groups, group_size, gate_first, shared_weight, gate_sigmoid, eps};
  const size_t a = is_f32 ? 16 : 8;
  const bool vec = group_size % 4 == 0 && y_stride % 4 == 0 && gate_stride % 4 == 0 && out_stride % 4 == 0 && aligned_to(y, a) &&
                   aligned_to(gate, a) && aligned_to(out, a) && aligned_to(weight, 16);
  hipStream_t st = as_stream(stream);
  if (is_f32) vec ? launch_gated<float, 4>(p, st) : launch_gated<float, 1>(p, st);
  else vec ? launch_gated<uint16_t, 4>(p, st) : launch_gated<uint16_t, 1>(p, st);
  SGL_CHECK_LAUNCH("gated_rmsnorm");
  return 0;
}

int sgl_amd_gate_mul(int is_f32, const void* gate, const void* up, void* out, int64_t rows, int d, int64_t in_stride, int64_t out_stride,
                     int glu_kind, float glu_limit, float glu_alpha, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(glu_kind > kGluNone && glu_kind < kGluKinds, "gate_mul: no activation %d", glu_kind);
  const GluParams act{glu_kind, glu_limit, glu_alpha};
  SGL_CHECK_ARG(gate && up && out && d > 0, "gate_mul: null operand or empty rows");
  SGL_CHECK_ARG(rows <= 65535, "gate_mul: at most 65535 rows per call (got %lld)", (long long)rows);
  if (rows <= 0) return 0;
  const dim3 grid((d + 255) / 256, static_cast<unsigned>(rows));
  if (is_f32)
    hipLaunchKernelGGL((gate_mul_kernel<float>), grid, dim3(256), 0, as_stream(stream), static_cast<const float*>(gate),
                       static_cast<const float*>(up), static_cast<float*>(out), d, in_stride, out_stride, act);
  else
    hipLaunchKernelGGL((gate_mul_kernel<uint16_t>), grid, dim3(256), 0, as_stream(stream), static_cast<const uint16_t*>(gate),
                       static_cast<const uint16_t*>(up), static_cast<uint16_t*>(out), d, in_stride, out_stride, act);
  SGL_CHECK_LAUNCH("gate_mul");
  return 0;
}

int sgl_amd_squared_relu(int is_f32, const void* in, void* out, int64_t rows, int d, int64_t in_stride, int64_t out_stride, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(in && out && d > 0, "squared_relu: null operand or empty rows");
  if (rows <= 0) return 0;
  if (is_f32) launch_squared_relu<float>(in, out, rows, d, in_stride, out_stride, as_stream(stream));
  else launch_squared_relu<uint16_t>(in, out, rows, d, in_stride, out_stride, as_stream(stream));
  SGL_CHECK_LAUNCH("squared_relu");
  return 0;
}

}  // extern "C"
