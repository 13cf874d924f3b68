// Router and the plain form of routed experts.
//
//   moe_route     logits W h + b in fp32, the `top` largest per token, softmax over those alone; or sigmoid scores, chosen by score +
//                 correction among the best groups of experts, weighted by score * scale; or the same with the softmax over all logits as the
//                 scores.  Experts from `real` on have no weights: their id is -1.  One more row may hold a gate: its sigmoid goes behind the
//                 weights.  bf16 rows: matrix instructions over
//                 slices of the columns, one wave each (a compute unit alone streams the router's rows far too slowly), then a
//                 launch that adds the slices and the bias and picks; fp32 rows and odd sizes: plain sums and the pick in one launch
//   experts_up / experts_down   act(gate h, up h) or act(up h), and the down projection, per (token, expert) pair for fp32 rows and sizes
//                 outside the grouped matrix kernels' forms: a wave sums one output; a pair with a negative expert is left out
#include "elem_io.hpp"
#include "glu.hpp"
#include "mfma_tiles.hpp"
#include "sglang_amd.h"

using namespace sgl_amd;

namespace {

struct RouteParams {
  const void* h;          // [tokens, K]
  int64_t h_stride;
  const void* w;          // [experts, K], rows contiguous
  const float* bias;      // [experts], or null
  float* weights;         // [tokens, top (+ 1 with a gate row)]
  int32_t* ids;           // [tokens, top]
  float* part;            // [slices, tokens, pad] partial logits
  int64_t tokens;
  int K, experts, top, slices, pad;
  int kind;               // 0: softmax over the chosen logits; scores: 1 sigmoid, 2 softmax over all logits
  const float* correction;// scores: [experts] added to them for the choice alone, or null
  int group_size, groups, keep;   // scores: equal groups of neighbours, experts of the best `keep` can be chosen
  int group_best;         // a group counts by 1: its best, 2: the sum of its two best
  int real, gate_row, w_stride;   // experts below `real` have weights; a row behind the experts' is a gate; columns of `weights`
  float scale;
};

__device__ __forceinline__ void wave_lds_fence() {     // (a wave's own array: LDS serves a wave in order)
  asm volatile("" ::: "memory");
  __builtin_amdgcn_wave_barrier();
}

// Scores: s[j] of expert lane + 64 j, z[j] what it is chosen by (-inf: not at all).  all, group: [64 N] of this wave.
template <int N>
__device__ __forceinline__ void score_experts(const RouteParams& p, float (&z)[N], float (&s)[N], int lane, float* all, float* group) {
  float top = -INFINITY;
#pragma unroll
  for (int j = 0; j < N; ++j) {
    if (p.kind == 1) s[j] = sigmoid_f(z[j]);
    else top = fmaxf(top, lane + 64 * j < p.experts ? z[j] : -INFINITY);
  }
  if (p.kind == 2) {
    top = wave_max(top);
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < N; ++j) {
      s[j] = lane + 64 * j < p.experts ? expf(z[j] - top) : 0.f;
      sum += s[j];
    }
    sum = wave_sum(sum);
#pragma unroll
    for (int j = 0; j < N; ++j) s[j] /= sum;
  }
#pragma unroll
  for (int j = 0; j < N; ++j) {
    const int e = lane + 64 * j;
    z[j] = e < p.experts ? s[j] + (p.correction ? p.correction[e] : 0.f) : -INFINITY;
    if (!(z[j] == z[j])) z[j] = -INFINITY;
    all[e] = z[j];
  }
  if (p.keep >= p.groups) return;
  wave_lds_fence();
  for (int g = lane; g < p.groups; g += 64) {
    float a = -INFINITY, b = -INFINITY;                // the two largest
    for (int i = 0; i < p.group_size; ++i) {
      const float v = all[g * p.group_size + i];
      b = fmaxf(b, fminf(a, v));
      a = fmaxf(a, v);
    }
    group[g] = p.group_size > 1 && p.group_best == 2 ? a + b : a;
  }
  wave_lds_fence();
#pragma unroll
  for (int j = 0; j < N; ++j) {
    const int e = lane + 64 * j;
    if (e >= p.experts) continue;
    const int g = e / p.group_size;
    const float mine = group[g];
    int ahead = 0;
    for (int i = 0; i < p.groups; ++i) ahead += group[i] > mine || (group[i] == mine && i < g) ? 1 : 0;
    if (ahead >= p.keep) z[j] = -INFINITY;
  }
  wave_lds_fence();
}

// A wave picks for one token: z[j] is the logit of expert lane + 64 j.  An expert's place is the number of experts in front of it
// (larger logit, or the same and a smaller index; what is not a number goes last), so every place has exactly one expert.
template <int N>
__device__ __forceinline__ void pick_experts(const RouteParams& p, int64_t t, float (&z)[N], int lane, float* all) {
  int place[N];
  float top = -INFINITY, score[N];
  if (p.gate_row) {
#pragma unroll
    for (int j = 0; j < N; ++j)
      if (lane + 64 * j == p.experts) p.weights[t * p.w_stride + p.top] = sigmoid_f(z[j]);
  }
  if (p.kind) score_experts<N>(p, z, score, lane, all, all + 64 * N);
#pragma unroll
  for (int j = 0; j < N; ++j) {
    place[j] = 0;
    if (!(z[j] == z[j]) || lane + 64 * j >= p.experts) z[j] = -INFINITY;
    top = fmaxf(top, z[j]);
    all[lane + 64 * j] = z[j];
  }
  top = wave_max(top);
  wave_lds_fence();
#pragma unroll
  for (int i = 0; i < N; ++i) {
    const int n = p.experts - 64 * i < 64 ? p.experts - 64 * i : 64;
#pragma unroll 4
    for (int l = 0; l < n; l += 4) {                   // (what lies behind the last expert is -inf, in front of nobody)
      float other[4];
      ld4(all + 64 * i + l, other);
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int j = 0; j < N; ++j) place[j] += other[u] > z[j] || (other[u] == z[j] && (i < j || (i == j && l + u < lane))) ? 1 : 0;
    }
  }
  float e[N], sum = 0.f;
#pragma unroll
  for (int j = 0; j < N; ++j) {
    const bool taken = place[j] < p.top && lane + 64 * j < p.experts;
    e[j] = taken ? (p.kind ? score[j] * p.scale : expf(z[j] - top)) : 0.f;
    sum += e[j];
  }
  sum = p.kind ? 1.0f : wave_sum(sum);
#pragma unroll
  for (int j = 0; j < N; ++j)
    if (place[j] < p.top && lane + 64 * j < p.experts) {
      p.weights[t * p.w_stride + place[j]] = e[j] / sum;
      p.ids[t * p.top + place[j]] = lane + 64 * j < p.real ? lane + 64 * j : -1;
    }
}

// One wave: 16 MT tokens, 16 NT experts (all of them), one slice of the columns.
template <int NT, int MT>
__global__ __launch_bounds__(64) void moe_route_slice_kernel(RouteParams p) {
  constexpr int kSteps = NT * MT <= 8 ? 4 : NT * MT <= 16 ? 2 : 1;       // column steps in flight together
  const int lane = threadIdx.x, i16 = lane & 15, g = lane >> 4;
  const int64_t t0 = static_cast<int64_t>(blockIdx.x) * (16 * MT);
  const int chunk = ((p.K + p.slices - 1) / p.slices + 31) / 32 * 32, k_first = blockIdx.y * chunk;
  const int k_end = k_first + chunk < p.K ? k_first + chunk : p.K;
  const uint16_t *hr[MT], *wr[NT];
  const int rows = p.experts + p.gate_row;
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int64_t t = t0 + 16 * m + i16;
    hr[m] = static_cast<const uint16_t*>(p.h) + (t < p.tokens ? t : p.tokens - 1) * p.h_stride;
  }
#pragma unroll
  for (int n = 0; n < NT; ++n) {
    const int e = 16 * n + i16;
    wr[n] = static_cast<const uint16_t*>(p.w) + static_cast<int64_t>(e < rows ? e : rows - 1) * p.K;
  }
  f32x4_t acc[NT][MT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int m = 0; m < MT; ++m) acc[n][m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = k_first; k0 < k_end; k0 += kSteps * 32) {
    U4 x[kSteps][MT], w[kSteps][NT];
#pragma unroll
    for (int s = 0; s < kSteps; ++s) {
      const int k = k0 + 32 * s + 8 * g;
      const bool in = k < k_end;
#pragma unroll
      for (int m = 0; m < MT; ++m) x[s][m] = keep_if(ld16(in ? hr[m] + k : hr[m]), in);
#pragma unroll
      for (int n = 0; n < NT; ++n) w[s][n] = ld16(in ? wr[n] + k : wr[n]);
    }
#pragma unroll
    for (int s = 0; s < kSteps; ++s)
#pragma unroll
      for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < MT; ++m) acc[n][m] = mfma_bf16(as_frag(w[s][n]), as_frag(x[s][m]), acc[n][m]);
  }
  // lane: token 16 m + i16, experts 16 n + 4 g + r
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int64_t t = t0 + 16 * m + i16;
    if (t >= p.tokens) continue;
    float* dst = p.part + (blockIdx.y * p.tokens + t) * p.pad + 4 * g;
#pragma unroll
    for (int n = 0; n < NT; ++n) *reinterpret_cast<f32x4_t*>(dst + 16 * n) = acc[n][m];
  }
}

// A wave per token.
template <int N>
__global__ __launch_bounds__(256) void moe_route_pick_kernel(RouteParams p) {
  __shared__ __attribute__((aligned(16))) float all[4][2 * N * 64];
  const int lane = threadIdx.x & 63;
  const int64_t t = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
  if (t >= p.tokens) return;
  float z[N];
#pragma unroll
  for (int j = 0; j < N; ++j) {
    const int e = lane + 64 * j;
    z[j] = -INFINITY;
    if (e < p.experts + p.gate_row) {
      float v = p.bias && e < p.experts ? p.bias[e] : 0.f;
#pragma unroll 4
      for (int s = 0; s < p.slices; ++s) v += p.part[(s * p.tokens + t) * p.pad + e];
      z[j] = v;
    }
  }
  pick_experts<N>(p, t, z, lane, all[threadIdx.x >> 6]);
}

// One token a workgroup, a wave per expert in turn.
template <typename T>
__global__ __launch_bounds__(256) void moe_route_plain_kernel(RouteParams p) {
  __shared__ float logits[256];
  __shared__ __attribute__((aligned(16))) float all[512];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t t = blockIdx.x;
  const T* hr = static_cast<const T*>(p.h) + t * p.h_stride;
  for (int e = wave; e < p.experts + p.gate_row; e += 4) {
    const T* wr = static_cast<const T*>(p.w) + static_cast<int64_t>(e) * p.K;
    float s = 0.f;
    for (int k = lane; k < p.K; k += 64) s += ld1(hr + k) * ld1(wr + k);
    s = wave_sum(s);
    if (lane == 0) logits[e] = s + (p.bias && e < p.experts ? p.bias[e] : 0.f);
  }
  __syncthreads();
  if (wave == 0) {
    float z[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) z[j] = lane + 64 * j < p.experts + p.gate_row ? logits[lane + 64 * j] : -INFINITY;
    pick_experts<4>(p, t, z, lane, all);
  }
}

template <int NT>
void launch_route(const RouteParams& p, hipStream_t st) {
  constexpr int MT = NT <= 8 ? 4 : 2;
  const dim3 grid(static_cast<unsigned>((p.tokens + 16 * MT - 1) / (16 * MT)), p.slices);
  if (p.tokens <= 16) hipLaunchKernelGGL((moe_route_slice_kernel<NT, 1>), dim3(1, p.slices), dim3(64), 0, st, p);
  else hipLaunchKernelGGL((moe_route_slice_kernel<NT, MT>), grid, dim3(64), 0, st, p);
  hipLaunchKernelGGL((moe_route_pick_kernel<(NT + 3) / 4>), dim3(static_cast<unsigned>((p.tokens + 3) / 4)), dim3(256), 0, st, p);
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
  GluParams glu;
};

// kUp: with the activation, kGated: of gate rows and up rows
template <typename T, bool kUp, bool kGated>
__global__ __launch_bounds__(256) void experts_plain_kernel(ExpertParams p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int64_t i = blockIdx.x;
  const int e = p.ids[i];
  if (e < 0 || e >= p.experts) return;
  const T* x = static_cast<const T*>(p.x) + i / p.div * p.x_stride;
  const T* w = static_cast<const T*>(p.w) + static_cast<int64_t>(e) * p.N * (kGated ? 2 : 1) * p.K;
  for (int n = blockIdx.y * 32 + wave; n < p.N && n < static_cast<int>(blockIdx.y) * 32 + 32; n += 4) {
    const T *w0 = w + static_cast<int64_t>(n) * p.K, *w1 = w0 + static_cast<int64_t>(p.N) * p.K;
    float a = 0.f, u = 0.f;
    for (int k = lane; k < p.K; k += 64) {
      const float v = ld1(x + k);
      a += v * ld1(w0 + k);
      if (kGated) u += v * ld1(w1 + k);
    }
    a = wave_sum(a);
    if (kGated) a = glu<false>(p.glu, a, wave_sum(u));
    else if (kUp) a = squared_relu(a);
    if (lane == 0) st1(static_cast<T*>(p.out) + i * p.o_stride + n, a);
  }
}

}  // namespace

extern "C" {

int sgl_amd_moe_route(int is_f32, const void* h, int64_t h_stride, const void* w, const float* bias, float* topk_weights, int32_t* topk_ids,
                      float* partials, int slices, int pad, int64_t tokens, int K, int experts, int top, int kind, const float* correction,
                      int groups, int keep, int group_best, float scale, int real, int gate_row, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(h && w && topk_weights && topk_ids && K > 0, "moe_route: null operand");
  SGL_CHECK_ARG(kind >= 0 && kind <= 2 && (group_best == 1 || group_best == 2) && real >= 0 && real <= experts && (gate_row == 0 || gate_row == 1) &&
                    experts + gate_row <= 256, "moe_route: scores %d, %d of %d experts with weights, gate row %d", kind, real, experts, gate_row);
  SGL_CHECK_ARG(experts >= 1 && experts <= 256 && top >= 1 && top <= experts && top <= 64, "moe_route: %d of %d experts (at most 64 of 256)", top, experts);
  SGL_CHECK_ARG(tokens <= 0x7fffffffLL, "moe_route: too many tokens");
  SGL_CHECK_ARG(!kind || (groups >= 1 && experts % groups == 0 && keep >= 1 && keep <= groups && top <= keep * (experts / groups)),
                "moe_route: %d of %d experts from %d of %d groups", top, experts, keep, groups);
  if (tokens <= 0) return 0;
  RouteParams p{h, h_stride, w, bias, topk_weights, topk_ids, partials, tokens, K, experts, top, slices, pad,
                kind, correction, kind ? experts / groups : experts, kind ? groups : 1, kind ? keep : 1, group_best, real, gate_row, top + gate_row, scale};
  hipStream_t st = as_stream(stream);
  if (partials) {
    const int nt = pad / 16;
    SGL_CHECK_ARG(!is_f32 && K % 8 == 0 && h_stride % 8 == 0 && aligned_to(h, 16) && aligned_to(w, 16) && aligned_to(partials, 16),
                  "moe_route: the matrix form takes bf16 rows of whole 16-byte vectors");
    SGL_CHECK_ARG(pad % 16 == 0 && (nt & (nt - 1)) == 0 && nt >= 1 && nt <= 16 && pad >= experts + gate_row && slices >= 1 && slices <= 65535,
                  "moe_route: %d slices of %d columns for %d experts", slices, pad, experts);
    if (nt == 1) launch_route<1>(p, st);
    else if (nt == 2) launch_route<2>(p, st);
    else if (nt == 4) launch_route<4>(p, st);
    else if (nt == 8) launch_route<8>(p, st);
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
                          int64_t pairs, int top, int N, int K, int experts, int glu_kind, float glu_limit, float glu_alpha, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(!up || (glu_kind > kGluNone && glu_kind < kActKinds), "experts_plain: no activation %d", glu_kind);
  SGL_CHECK_ARG(x && w && ids && out && N > 0 && K > 0 && experts > 0 && top > 0 && pairs <= 0x7fffffffLL && (N + 31) / 32 <= 65535,
                "experts_plain: %d experts of %d x %d", experts, N, K);
  if (pairs <= 0) return 0;
  ExpertParams p{x, x_stride, w, ids, out, o_stride, N, K, experts, up ? top : 1, GluParams{glu_kind, glu_limit, glu_alpha}};
  const dim3 grid(static_cast<unsigned>(pairs), (N + 31) / 32);
  hipStream_t st = as_stream(stream);
  const bool gated = up && act_gated(glu_kind);
  if (is_f32) {
    if (gated) hipLaunchKernelGGL((experts_plain_kernel<float, true, true>), grid, dim3(256), 0, st, p);
    else if (up) hipLaunchKernelGGL((experts_plain_kernel<float, true, false>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((experts_plain_kernel<float, false, false>), grid, dim3(256), 0, st, p);
  } else {
    if (gated) hipLaunchKernelGGL((experts_plain_kernel<uint16_t, true, true>), grid, dim3(256), 0, st, p);
    else if (up) hipLaunchKernelGGL((experts_plain_kernel<uint16_t, true, false>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((experts_plain_kernel<uint16_t, false, false>), grid, dim3(256), 0, st, p);
  }
  SGL_CHECK_LAUNCH("experts_plain");
  return 0;
}

}  // extern "C"
