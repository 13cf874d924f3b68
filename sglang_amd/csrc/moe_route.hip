// Router and the plain form of routed experts.
//
//   moe_route     logits W h + b in fp32, the `top` largest per token, softmax over those alone: one launch, so the logits never
//                 leave the workgroup (bf16 rows on matrix instructions, fp32 rows and odd sizes by plain sums)
//   experts_up / experts_down   silu(gate h) * (up h) and its down projection per (token, expert) pair for fp32 rows and sizes outside
//                 the grouped matrix kernels' forms: a wave sums one output
#include "elem_io.hpp"
#include "mfma_tiles.hpp"
#include "sglang_amd.h"

using namespace sgl_amd;

namespace {

struct RouteParams {
  const void* h;          // [tokens, K]
  int64_t h_stride;
  const void* w;          // [experts, K], rows contiguous
  const float* bias;      // [experts], or null
  float* weights;         // [tokens, top]
  int32_t* ids;           // [tokens, top]
  int64_t tokens;
  int K, experts, top;
};

// A wave picks for one token: z[j] is the logit of expert lane + 64 j (-inf behind the last).
template <int N>
__device__ __forceinline__ void pick_experts(const RouteParams& p, int64_t t, float (&z)[N], int lane) {
  float mine = -INFINITY, best = 0.f, sum = 0.f;
  int my_id = 0;
  for (int i = 0; i < p.top; ++i) {
    float bv = -INFINITY;
    int be = 0x7fffffff;
#pragma unroll
    for (int j = 0; j < N; ++j)
      if (lane + 64 * j < p.experts && (be == 0x7fffffff || z[j] > bv) && z[j] > -INFINITY) { bv = z[j]; be = lane + 64 * j; }
    for (int off = 32; off > 0; off >>= 1) {
      const float ov = __shfl_xor(bv, off, 64);
      const int oe = __shfl_xor(be, off, 64);
      if (oe != 0x7fffffff && (be == 0x7fffffff || ov > bv || (ov == bv && oe < be))) { bv = ov; be = oe; }
    }
    if (be == 0x7fffffff) { be = i; bv = -INFINITY; }  // (logits that are not numbers: some expert, weight zero or not a number)
#pragma unroll
    for (int j = 0; j < N; ++j)
      if (be == lane + 64 * j) z[j] = -INFINITY;
    if (i == 0) best = bv;
    if (lane == i) { mine = bv; my_id = be; }
    sum += expf(bv - best);
  }
  if (lane < p.top) {
    p.weights[t * p.top + lane] = expf(mine - best) / sum;
    p.ids[t * p.top + lane] = my_id;
  }
}

// 16 tokens a workgroup; its kWaves waves share the columns, partial logits meet in LDS, then a wave picks for one token at a time.
template <int NT, int kWaves>
__global__ __launch_bounds__(kWaves * 64) void moe_route_mfma_kernel(RouteParams p) {
  constexpr int LS = NT * 16 + 4;                    // logits of a token, in fp32
  __shared__ __attribute__((aligned(16))) float part[(kWaves > 4 ? 4 : kWaves)][16][LS];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), i16 = lane & 15, g = lane >> 4;
  const int64_t t0 = static_cast<int64_t>(blockIdx.x) * 16;
  const int64_t t = t0 + i16 < p.tokens ? t0 + i16 : p.tokens - 1;
  const uint16_t* hr = static_cast<const uint16_t*>(p.h) + t * p.h_stride;
  const uint16_t* wr[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int e = 16 * n + i16;
    wr[n] = static_cast<const uint16_t*>(p.w) + static_cast<int64_t>(e < p.experts ? e : p.experts - 1) * p.K;
  }
  f32x4_t acc[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n) acc[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = wave * 32; k0 < p.K; k0 += kWaves * 32) {
    const int k = k0 + 8 * g;
    const bool in = k < p.K;
    const bf16x8_t x = as_frag(keep_if(ld16(in ? hr + k : hr), in));
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[n] = mfma_bf16(as_frag(ld16(in ? wr[n] + k : wr[n])), x, acc[n]);
  }
  // lane: token i16, experts 16 n + 4 g + r.  Four slabs: with more waves they add up in turn
#pragma unroll
  for (int turn = 0; turn < (kWaves + 3) / 4; ++turn) {
    if (wave / 4 == turn) {
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        f32x4_t* dst = reinterpret_cast<f32x4_t*>(&part[wave & 3][i16][16 * n + 4 * g]);
        *dst = turn == 0 ? acc[n] : *dst + acc[n];
      }
    }
    __syncthreads();
  }
  constexpr int PN = (NT + 3) / 4;
  for (int tk = wave; tk < 16 && t0 + tk < p.tokens; tk += kWaves) {
    float z[PN];
#pragma unroll
    for (int j = 0; j < PN; ++j) {
      const int e = lane + 64 * j;
      z[j] = -INFINITY;
      if (e < p.experts) {
        float v = p.bias ? p.bias[e] : 0.f;
#pragma unroll
        for (int s = 0; s < (kWaves > 4 ? 4 : kWaves); ++s) v += part[s][tk][e];
        z[j] = v;
      }
    }
    pick_experts<PN>(p, t0 + tk, z, lane);
  }
}

// One token a workgroup, a wave per expert in turn.
template <typename T>
__global__ __launch_bounds__(256) void moe_route_plain_kernel(RouteParams p) {
  __shared__ float logits[256];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t t = blockIdx.x;
  const T* hr = static_cast<const T*>(p.h) + t * p.h_stride;
  for (int e = wave; e < p.experts; e += 4) {
    const T* wr = static_cast<const T*>(p.w) + static_cast<int64_t>(e) * p.K;
    float s = 0.f;
    for (int k = lane; k < p.K; k += 64) s += ld1(hr + k) * ld1(wr + k);
    s = wave_sum(s);
    if (lane == 0) logits[e] = s + (p.bias ? p.bias[e] : 0.f);
  }
  __syncthreads();
  if (wave == 0) {
    float z[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) z[j] = lane + 64 * j < p.experts ? logits[lane + 64 * j] : -INFINITY;
    pick_experts<4>(p, t, z, lane);
  }
}

template <int NT>
void launch_route(const RouteParams& p, hipStream_t st) {
  const dim3 grid(static_cast<unsigned>((p.tokens + 15) / 16));
  if (p.tokens <= 2048 && p.K >= 1024) hipLaunchKernelGGL((moe_route_mfma_kernel<NT, 16>), grid, dim3(1024), 0, st, p);
  else hipLaunchKernelGGL((moe_route_mfma_kernel<NT, 4>), grid, dim3(256), 0, st, p);
}

// ---------------------------------------------------------------------------------------------------------------
struct ExpertParams {
  const void* x;          // up: [tokens, K] (pair i reads row i / top), down: [pairs, K]
  int64_t x_stride;
  const void* w;          // up: [experts, 2 N, K] gate rows, then up rows; down: [experts, N, K]
  const int32_t* ids;     // [pairs]
  void* out;              // [pairs, N]
  int64_t o_stride;
  int N, K, experts, div;
};

template <typename T, bool kUp>
__global__ __launch_bounds__(256) void experts_plain_kernel(ExpertParams p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t i = blockIdx.x;
  const int e = p.ids[i];
  if (e < 0 || e >= p.experts) return;
  const T* x = static_cast<const T*>(p.x) + i / p.div * p.x_stride;
  const T* w = static_cast<const T*>(p.w) + static_cast<int64_t>(e) * p.N * (kUp ? 2 : 1) * p.K;
  for (int n = blockIdx.y * 32 + wave; n < p.N && n < static_cast<int>(blockIdx.y) * 32 + 32; n += 4) {
    const T *w0 = w + static_cast<int64_t>(n) * p.K, *w1 = w0 + static_cast<int64_t>(p.N) * p.K;
    float a = 0.f, u = 0.f;
    for (int k = lane; k < p.K; k += 64) {
      const float v = ld1(x + k);
      a += v * ld1(w0 + k);
      if (kUp) u += v * ld1(w1 + k);
    }
    a = wave_sum(a);
    if (kUp) a = silu_f(a) * wave_sum(u);
    if (lane == 0) st1(static_cast<T*>(p.out) + i * p.o_stride + n, a);
  }
}

}  // namespace

extern "C" {

int sgl_amd_moe_route(int is_f32, const void* h, int64_t h_stride, const void* w, const float* bias, float* topk_weights, int32_t* topk_ids,
                      int64_t tokens, int K, int experts, int top, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(h && w && topk_weights && topk_ids && K > 0, "moe_route: null operand");
  SGL_CHECK_ARG(experts >= 1 && experts <= 256 && top >= 1 && top <= experts && top <= 64, "moe_route: %d of %d experts (at most 64 of 256)", top, experts);
  SGL_CHECK_ARG(tokens <= 0x7fffffffLL, "moe_route: too many tokens");
  if (tokens <= 0) return 0;
  RouteParams p{h, h_stride, w, bias, topk_weights, topk_ids, tokens, K, experts, top};
  hipStream_t st = as_stream(stream);
  if (!is_f32 && K % 8 == 0 && h_stride % 8 == 0 && aligned_to(h, 16) && aligned_to(w, 16)) {
    if (experts <= 16) launch_route<1>(p, st);
    else if (experts <= 32) launch_route<2>(p, st);
    else if (experts <= 64) launch_route<4>(p, st);
    else if (experts <= 128) launch_route<8>(p, st);
    else launch_route<16>(p, st);
  } else {
    const dim3 grid(static_cast<unsigned>(tokens));
    if (is_f32) hipLaunchKernelGGL((moe_route_plain_kernel<float>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((moe_route_plain_kernel<uint16_t>), grid, dim3(256), 0, st, p);
  }
  SGL_CHECK_LAUNCH("moe_route");
  return 0;
}

int sgl_amd_experts_plain(int is_f32, int up, const void* x, int64_t x_stride, const void* w, const int32_t* ids, void* out, int64_t o_stride,
                          int64_t pairs, int top, int N, int K, int experts, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(x && w && ids && out && N > 0 && K > 0 && experts > 0 && top > 0 && pairs <= 0x7fffffffLL && (N + 31) / 32 <= 65535,
                "experts_plain: %d experts of %d x %d", experts, N, K);
  if (pairs <= 0) return 0;
  ExpertParams p{x, x_stride, w, ids, out, o_stride, N, K, experts, up ? top : 1};
  const dim3 grid(static_cast<unsigned>(pairs), (N + 31) / 32);
  hipStream_t st = as_stream(stream);
  if (is_f32) {
    if (up) hipLaunchKernelGGL((experts_plain_kernel<float, true>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((experts_plain_kernel<float, false>), grid, dim3(256), 0, st, p);
  } else {
    if (up) hipLaunchKernelGGL((experts_plain_kernel<uint16_t, true>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((experts_plain_kernel<uint16_t, false>), grid, dim3(256), 0, st, p);
  }
  SGL_CHECK_LAUNCH("experts_plain");
  return 0;
}

}  // extern "C"
