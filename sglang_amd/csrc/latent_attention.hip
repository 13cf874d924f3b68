// Latent attention (one normed latent + one rotated key part cached per token, shared by all heads) over a paged pool.
//
//   latent_prepare         RMS norm of the latent, rotation of the key part and of every query head's rotated part, and the
//                          store of the cache row
//   head_gemm              per-head products  out[t, h, :] = w[h] x[t, h, :]  (absorbing the key up-projection into the query,
//                          expanding the attended latent into the value)
//   latent_attention       absorbed form: score = q_c . c + q_r . k_r, output = sum of latents; any token mix, any sizes, with
//                          an MFMA form for the sizes real models have and a plain form (every size, bf16 and fp32)
//
// A cache row is [rank latents | rot rotated] padded with zeros to a multiple of 32 elements; the pool is created zeroed and
// only the first rank + rot elements are ever written.
#include "elem_io.hpp"
#include "mfma_tiles.hpp"
#include "sglang_amd.h"

using namespace sgl_amd;

namespace {

struct PrepareParams {
  void* q;                   // [tokens, heads, dim + rot]: the last rot of every head are rotated in place
  int64_t q_stride;
  const void* dkv;           // [tokens, rank + rot]
  int64_t dkv_stride;
  const float* norm_w;       // [rank]
  const float* cos_sin;      // [positions, dims]: cos (dims / 2) | sin (dims / 2)
  const int64_t* positions;
  const int64_t* loc;
  void* cache;               // [slots, row]
  int64_t cache_stride;
  int heads, dim, rot, rot_dims, rank;
  int64_t max_pos;
  float eps;
  int vec;                   // rows of whole 4-element pieces, rot_dims == rot
};

template <typename T>
__global__ __launch_bounds__(256) void latent_prepare_kernel(PrepareParams p) {
  __shared__ float scratch[16];
  const int64_t t = blockIdx.x;
  int64_t pos = p.positions[t];
  if (pos >= p.max_pos) pos = p.max_pos - 1;      // (the host never passes one)
  const float* cs = p.cos_sin + pos * p.rot_dims;
  const int half = p.rot_dims >> 1;
  const T* src = static_cast<const T*>(p.dkv) + t * p.dkv_stride;
  T* dst = static_cast<T*>(p.cache) + p.loc[t] * p.cache_stride;
  float ss = 0.f;
  if (p.vec && p.rank <= 1024) {
    float v[4] = {0.f, 0.f, 0.f, 0.f}, w[4];
    const int c = threadIdx.x * 4;
    if (c < p.rank) { ld4(src + c, v); ld4(p.norm_w + c, w); }
    const float rs = 1.0f / sqrtf(block_sum(v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3], scratch) / static_cast<float>(p.rank) + p.eps);
    if (c < p.rank) {
      const float o[4] = {v[0] * rs * w[0], v[1] * rs * w[1], v[2] * rs * w[2], v[3] * rs * w[3]};
      st4(dst + c, o);
    }
  } else {
    for (int c = threadIdx.x; c < p.rank; c += 256) { const float v = ld1(src + c); ss += v * v; }
    const float rs = 1.0f / sqrtf(block_sum(ss, scratch) / static_cast<float>(p.rank) + p.eps);
    for (int c = threadIdx.x; c < p.rank; c += 256) st1(dst + c, ld1(src + c) * rs * p.norm_w[c]);
  }
  T* qt = static_cast<T*>(p.q) + t * p.q_stride;
  if (p.vec) {
    // two pairs a piece; every dimension of the rotated part turns
    const int per = p.rot >> 2;
    for (int idx = threadIdx.x; idx < (p.heads + 1) * per; idx += 256) {
      const int h = idx / per, i = (idx - h * per) * 2;
      const bool key = h == p.heads;
      T* qh = qt + static_cast<int64_t>(h) * (p.dim + p.rot) + p.dim + 2 * i;
      float v[4], o[4];
      ld4(key ? src + p.rank + 2 * i : qh, v);
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const float c = cs[i + j], s = cs[half + i + j];
        o[2 * j] = v[2 * j] * c - v[2 * j + 1] * s;
        o[2 * j + 1] = v[2 * j + 1] * c + v[2 * j] * s;
      }
      st4(key ? dst + p.rank + 2 * i : qh, o);
    }
    return;
  }
  // rotated parts: item = (head or the shared key, pair); dimensions beyond rot_dims pass unchanged
  const int pairs = (p.rot + 1) >> 1;
  for (int idx = threadIdx.x; idx < (p.heads + 1) * pairs; idx += 256) {
    const int h = idx / pairs, i = idx - h * pairs;
    const bool key = h == p.heads;
    const T* in = key ? src + p.rank : qt + static_cast<int64_t>(h) * (p.dim + p.rot) + p.dim;
    T* out = key ? dst + p.rank : qt + static_cast<int64_t>(h) * (p.dim + p.rot) + p.dim;
    if (i < half) {
      const float u = ld1(in + 2 * i), v = ld1(in + 2 * i + 1), c = cs[i], s = cs[half + i];
      st1(out + 2 * i, u * c - v * s);
      st1(out + 2 * i + 1, v * c + u * s);
    } else if (key) {
      st1(out + 2 * i, ld1(in + 2 * i));
      if (2 * i + 1 < p.rot) st1(out + 2 * i + 1, ld1(in + 2 * i + 1));
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
// out[t, h, n] = sum_k w[h, n, k] x[t, h, k].  x / out rows are strided; w is [heads, N, K] with K contiguous.
struct HeadGemmParams {
  const void* x;
  int64_t x_token, x_head;
  const void* w;
  void* out;
  int64_t o_token, o_head;
  int64_t tokens;
  int N, K, vec_out;
};

template <typename T>
__global__ __launch_bounds__(256) void head_gemm_plain_kernel(HeadGemmParams p) {
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y;
  const T* x = static_cast<const T*>(p.x) + t * p.x_token + h * p.x_head;
  const T* w = static_cast<const T*>(p.w) + static_cast<int64_t>(h) * p.N * p.K;
  T* o = static_cast<T*>(p.out) + t * p.o_token + h * p.o_head;
  for (int n = blockIdx.z * 256 + threadIdx.x; n < p.N; n += gridDim.z * 256) {
    float acc = 0.f;
    for (int k = 0; k < p.K; ++k) acc += ld1(w + static_cast<int64_t>(n) * p.K + k) * ld1(x + k);
    st1(o + n, acc);
  }
}

// MFMA form (bf16, K a multiple of 8, 16-byte aligned rows): a workgroup owns 16 output rows of one head and MT x 16 tokens; its
// four waves take a quarter of K each, both operands straight from memory (16 bytes per lane, four steps in flight), and meet
// in LDS.
template <int MT>
__global__ __launch_bounds__(256) void head_gemm_mfma_kernel(HeadGemmParams p) {
  __shared__ f32x4_t part[4][MT][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int n0 = blockIdx.x * 16;
  const int h = blockIdx.y;
  const int64_t t0 = static_cast<int64_t>(blockIdx.z) * (MT * 16);
  const int n = n0 + i16 < p.N ? n0 + i16 : p.N - 1;
  const uint16_t* wr = static_cast<const uint16_t*>(p.w) + (static_cast<int64_t>(h) * p.N + n) * p.K;
  const uint16_t* xr[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    int64_t t = t0 + m * 16 + i16;
    if (t >= p.tokens) t = p.tokens - 1;
    xr[m] = static_cast<const uint16_t*>(p.x) + t * p.x_token + h * p.x_head;
  }
  f32x4_t acc[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) acc[m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int quarter = (p.K + 127) / 128 * 32;
  const int k_end = (wave + 1) * quarter < p.K ? (wave + 1) * quarter : p.K;
  for (int k0 = wave * quarter; k0 < k_end; k0 += 128) {
    U4 a[4], bq[4][MT];
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int k = k0 + 32 * s + g * 8;
      a[s] = U4{0, 0, 0, 0};
      if (k < k_end) a[s] = ld16(wr + k);
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        bq[s][m] = U4{0, 0, 0, 0};
        if (k < k_end) bq[s][m] = ld16(xr[m] + k);
      }
    }
#pragma unroll
    for (int s = 0; s < 4; ++s)
#pragma unroll
      for (int m = 0; m < MT; ++m) acc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_frag(a[s]), as_frag(bq[s][m]), acc[m], 0, 0, 0);
  }
#pragma unroll
  for (int m = 0; m < MT; ++m) part[wave][m][lane] = acc[m];
  __syncthreads();
  for (int m = wave; m < MT; m += 4) {
    const int64_t t = t0 + m * 16 + i16;
    if (t >= p.tokens) continue;
    const f32x4_t v = (part[0][m][lane] + part[1][m][lane]) + (part[2][m][lane] + part[3][m][lane]);
    uint16_t* o = static_cast<uint16_t*>(p.out) + t * p.o_token + h * p.o_head + n0 + g * 4;
    if (p.vec_out && n0 + g * 4 + 4 <= p.N) {
      const float e[4] = {v[0], v[1], v[2], v[3]};
      st4(o, e);
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (n0 + g * 4 + r < p.N) o[r] = f2bf(v[r]);
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------
struct LatentAttnParams {
  const void* qc;            // [tokens, heads, rank] absorbed queries
  int64_t qc_token, qc_head;
  const void* qr;            // [tokens, heads, rot] rotated queries
  int64_t qr_token, qr_head;
  const void* cache;         // [slots, row]
  int64_t cache_stride;
  const int32_t* req_to_token;
  int64_t r2t_stride;
  const int64_t* req;        // [segments] row of req_to_token
  const int32_t* tok_seg;    // [tokens] (null: token index)
  const int64_t* positions;  // [tokens]
  void* out;                 // [tokens, heads, rank]
  int64_t o_token, o_head;
  float* part_o;             // [tokens, heads, splits, rank] when splits > 1
  float* part_ml;            // [tokens, heads, splits, 2]
  int heads, rank, rot, window, splits;
  float scale;
  const float* sinks;        // [heads] scores in the softmax denominator that carry no value, or null
};

// 1 / denominator in units of e^m, for the sum l taken relative to the maximum m: a sink joins here
__device__ __forceinline__ float inverse_sum(float m, float l, const float* sinks, int head) {
  if (!sinks) return l > 0.f ? 1.0f / l : 0.f;
  const float s = sinks[head], top = fmaxf(m, s), f = expf(m - top);
  return f / (l * f + expf(s - top));
}

__device__ __forceinline__ void key_range(const LatentAttnParams& p, int64_t pos, int split, int& lo, int& hi) {
  const int first = p.window > 0 && pos + 1 > p.window ? static_cast<int>(pos + 1 - p.window) : 0;
  const int n = static_cast<int>(pos) + 1 - first;
  const int per = (n + p.splits - 1) / p.splits;
  lo = first + split * per;
  hi = lo + per < static_cast<int>(pos) + 1 ? lo + per : static_cast<int>(pos) + 1;
}

// One workgroup per (token, head, split): thread = key for the scores, thread = latent column for the sums.
template <typename T>
__global__ __launch_bounds__(256) void latent_attention_plain_kernel(LatentAttnParams p) {
  extern __shared__ float lds[];
  __shared__ float scratch[16];
  const int dk = p.rank + p.rot;
  float* q = lds;                 // [dk]
  float* acc = q + dk;            // [rank]
  float* sc = acc + p.rank;       // [256]
  int* slot = reinterpret_cast<int*>(sc + 256);   // [256]
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y, split = blockIdx.z;
  const int64_t b = p.tok_seg ? p.tok_seg[t] : t;
  const int32_t* row = p.req_to_token + p.req[b] * p.r2t_stride;
  const T* cache = static_cast<const T*>(p.cache);
  int lo, hi;
  key_range(p, p.positions[t], split, lo, hi);
  const T* qc = static_cast<const T*>(p.qc) + t * p.qc_token + h * p.qc_head;
  const T* qr = static_cast<const T*>(p.qr) + t * p.qr_token + h * p.qr_head;
  for (int c = threadIdx.x; c < dk; c += 256) q[c] = c < p.rank ? ld1(qc + c) : ld1(qr + c - p.rank);
  for (int c = threadIdx.x; c < p.rank; c += 256) acc[c] = 0.f;
  __syncthreads();
  float m = -INFINITY, l = 0.f;
  for (int j0 = lo; j0 < hi; j0 += 256) {
    const int j = j0 + threadIdx.x;
    float s = -INFINITY;
    int sl = 0;
    if (j < hi) {
      sl = row[j];
      const T* k = cache + static_cast<int64_t>(sl) * p.cache_stride;
      float d = 0.f;
      for (int c = 0; c < dk; ++c) d += q[c] * ld1(k + c);
      s = d * p.scale;
    }
    const float mn = fmaxf(m, block_max(s, scratch));
    const float e = j < hi ? expf(s - mn) : 0.f;
    const float fix = expf(m - mn);
    l = l * fix + block_sum(e, scratch);
    m = mn;
    sc[threadIdx.x] = e;
    slot[threadIdx.x] = sl;
    __syncthreads();
    const int n = hi - j0 < 256 ? hi - j0 : 256;
    for (int c = threadIdx.x; c < p.rank; c += 256) {
      float a = acc[c] * fix;
      for (int i = 0; i < n; ++i) a += sc[i] * ld1(cache + static_cast<int64_t>(slot[i]) * p.cache_stride + c);
      acc[c] = a;
    }
    __syncthreads();
  }
  if (p.splits == 1) {
    const float inv = inverse_sum(m, l, p.sinks, h);
    T* o = static_cast<T*>(p.out) + t * p.o_token + h * p.o_head;
    for (int c = threadIdx.x; c < p.rank; c += 256) st1(o + c, acc[c] * inv);
  } else {
    const int64_t slot_o = (t * p.heads + h) * p.splits + split;
    for (int c = threadIdx.x; c < p.rank; c += 256) p.part_o[slot_o * p.rank + c] = acc[c];
    if (threadIdx.x == 0) { p.part_ml[slot_o * 2] = m; p.part_ml[slot_o * 2 + 1] = l; }
  }
}

// Splits of one (token, head), VEC columns a thread.  An empty split has m = -inf, l = 0 and zero sums: its weight is 0.
template <typename T, int VEC>
__global__ __launch_bounds__(256) void latent_merge_kernel(LatentAttnParams p) {
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y;
  const int64_t base = (t * p.heads + h) * p.splits;
  const float* ml = p.part_ml + base * 2;
  float m = -INFINITY;
  for (int s = 0; s < p.splits; ++s) m = fmaxf(m, ml[s * 2]);
  for (int c = threadIdx.x * VEC; c < p.rank; c += blockDim.x * VEC) {
    float l = 0.f, a[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) a[j] = 0.f;
#pragma unroll 4
    for (int s = 0; s < p.splits; ++s) {
      const float w = expf(ml[s * 2] - m);
      float v[VEC];
      ldv<VEC>(p.part_o + (base + s) * p.rank + c, v);
      l += w * ml[s * 2 + 1];
#pragma unroll
      for (int j = 0; j < VEC; ++j) a[j] += w * v[j];
    }
    const float inv = inverse_sum(m, l, p.sinks, h);
#pragma unroll
    for (int j = 0; j < VEC; ++j) a[j] *= inv;
    stv<VEC>(static_cast<T*>(p.out) + t * p.o_token + h * p.o_head + c, a);
  }
}

template <typename T>
void launch_latent_merge(const LatentAttnParams& p, int64_t tokens, hipStream_t st) {
  const dim3 grid(static_cast<unsigned>(tokens), p.heads);
  const size_t al = sizeof(T) * 4;
  if (p.rank % 4 == 0 && p.o_token % 4 == 0 && p.o_head % 4 == 0 && aligned_to(p.out, al) && aligned_to(p.part_o, 16)) {
    const int threads = p.rank >= 1024 ? 256 : (p.rank / 4 + 63) / 64 * 64;
    hipLaunchKernelGGL((latent_merge_kernel<T, 4>), grid, dim3(threads), 0, st, p);
  } else {
    hipLaunchKernelGGL((latent_merge_kernel<T, 1>), grid, dim3(256), 0, st, p);
  }
}

// ---------------------------------------------------------------------------------------------------------------
// MFMA form of the absorbed attention (bf16).  A workgroup = one token, HG groups of 16 heads (four waves each), one key split;
// tiles of 64 keys are gathered once into LDS and serve both contractions of all groups, the next tile's rows waiting in
// registers meanwhile where they fit.
//   scores   wave w of a group: keys 16 w .. + 16 as the A operand, the group's queries (registers) as B -> lane holds head
//            lane & 15
//   weights  exp2 in fp32; kept to ~17 bits as a bf16 pair (high, rest), so the sum over values loses nothing to rounding
//   values   wave w owns a quarter of the latent columns: O^T = V^T P^T, the V^T operand from the row-major tile by
//            ds_read_b64_tr_b16; a lane's accumulators belong to one head, so the rescale factor is a lane scalar
constexpr int kTile = 64;

template <int KS, int OT, int HG>
__global__ __launch_bounds__(256 * HG, 2) void latent_attention_mfma_kernel(LatentAttnParams p) {
  extern __shared__ __attribute__((aligned(16))) uint16_t smem[];
  const int dk = (p.rank + p.rot + 31) & ~31;
  constexpr int ls = KS * 32 + 8;                              // columns dk .. KS * 32 are zero
  constexpr int PS = kTile + 8;
  constexpr int TPR = 4 * HG, kPieces = KS / HG;               // threads a row, 16-byte pieces a thread
  constexpr bool kAhead = kPieces <= 12;
  uint16_t* tile = smem;                                       // [64][ls]
  const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int lane = threadIdx.x & 63, wave = wid & 3, hg = wid >> 2, i16 = lane & 15, g = lane >> 4;
  uint16_t* ph = tile + kTile * ls + hg * 2 * 16 * PS;         // [16][PS] weights of this group, high part
  uint16_t* pl = ph + 16 * PS;                                 //          rest
  float* wmax = reinterpret_cast<float*>(tile + kTile * ls + HG * 2 * 16 * PS) + hg * 64;      // [4][16]
  const int64_t t = blockIdx.x;
  const int head = (blockIdx.y * HG + hg) * 16 + i16, split = blockIdx.z;
  const int hc = head < p.heads ? head : p.heads - 1;
  const int64_t b = p.tok_seg ? p.tok_seg[t] : t;
  const int32_t* row = p.req_to_token + p.req[b] * p.r2t_stride;
  const uint16_t* cache = static_cast<const uint16_t*>(p.cache);
  int lo, hi;
  key_range(p, p.positions[t], split, lo, hi);

  bf16x8_t q[KS];
  {
    const uint16_t* qc = static_cast<const uint16_t*>(p.qc) + t * p.qc_token + hc * p.qc_head;
    const uint16_t* qr = static_cast<const uint16_t*>(p.qr) + t * p.qr_token + hc * p.qr_head;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      // one load from a chosen address (no branch: all are in flight together), zero behind the last element
      const int c = 32 * k + 8 * g;
      const uint16_t* src = c < p.rank ? qc + c : c < p.rank + p.rot ? qr + (c - p.rank) : qc;
      U4 v = ld16(src);
      const uint32_t keep = c < p.rank + p.rot ? 0xffffffffu : 0u;
      v.x &= keep; v.y &= keep; v.z &= keep; v.w &= keep;
      q[k] = as_frag(v);
    }
  }
  f32x4_t o[OT];
#pragma unroll
  for (int i = 0; i < OT; ++i) o[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  const float sc = p.scale * kLog2e;
  // TPR threads a row (64 or 128 consecutive bytes a step); rows behind the last key are zero (finite, weight zero)
  const int r_row = threadIdx.x / TPR, r_col = (threadIdx.x % TPR) * 8;
  U4 piece[kPieces];
  bool have = false;
  int slot = lo + r_row < hi ? row[lo + r_row] : -1;
  auto fetch = [&]() __attribute__((always_inline)) {
    const uint16_t* src = cache + static_cast<int64_t>(slot < 0 ? 0 : slot) * p.cache_stride + r_col;
#pragma unroll
    for (int k = 0; k < kPieces; ++k) piece[k] = ld16(r_col + TPR * 8 * k < dk ? src + TPR * 8 * k : src);
    have = slot >= 0;
  };
  if (kAhead) fetch();
  for (int j0 = lo; j0 < hi; j0 += kTile) {
    const int n = hi - j0 < kTile ? hi - j0 : kTile;
    if (!kAhead) fetch();
#pragma unroll
    for (int k = 0; k < kPieces; ++k) {
      const uint32_t keep = have && r_col + TPR * 8 * k < dk ? 0xffffffffu : 0u;
      U4 v = piece[k];
      v.x &= keep; v.y &= keep; v.z &= keep; v.w &= keep;
      st16(tile + r_row * ls + r_col + TPR * 8 * k, v);
    }
    slot = j0 + kTile + r_row < hi ? row[j0 + kTile + r_row] : -1;
    __syncthreads();
    if (kAhead && j0 + kTile < hi) fetch();
    f32x4_t s = {0.f, 0.f, 0.f, 0.f}, s2 = {0.f, 0.f, 0.f, 0.f};
    {
      const uint16_t* kr = tile + (16 * wave + i16) * ls + 8 * g;
#pragma unroll
      for (int k = 0; k < KS; k += 2) {              // two chains: a product does not wait for the one before it
        s = mfma_bf16(as_frag(ld16(kr + 32 * k)), q[k], s);
        s2 = mfma_bf16(as_frag(ld16(kr + 32 * (k + 1))), q[k + 1], s2);
      }
      s += s2;
    }
    float mx = -INFINITY;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s[r] = 16 * wave + 4 * g + r < n ? s[r] * sc : -INFINITY;
      mx = fmaxf(mx, s[r]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (g == 0) wmax[wave * 16 + i16] = mx;
    __syncthreads();
    const float mn = fmaxf(fmaxf(fmaxf(wmax[i16], wmax[16 + i16]), fmaxf(wmax[32 + i16], wmax[48 + i16])), m);
    const float fix = fast_exp2(m - mn);
    m = mn;
    l *= fix;
    float hi_p[4], lo_p[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float e = fast_exp2(s[r] - mn);
      l += e;
      hi_p[r] = rbf(e);
      lo_p[r] = e - hi_p[r];
    }
    st4(ph + i16 * PS + 16 * wave + 4 * g, hi_p);
    st4(pl + i16 * PS + 16 * wave + 4 * g, lo_p);
    __syncthreads();
    bf16x8_t pf[2][2];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int w = 0; w < 2; ++w) {
        const uint16_t* pr = (w ? pl : ph) + i16 * PS + 32 * kk + 4 * g;
        const uint2 a = *reinterpret_cast<const uint2*>(pr), c = *reinterpret_cast<const uint2*>(pr + 16);
        pf[kk][w] = as_frag(U4{a.x, a.y, c.x, c.y});
      }
#pragma unroll
    for (int i = 0; i < OT; ++i) o[i] *= fix;
    // (columns behind the rank are computed and never stored)
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int i = 0; i < OT; ++i) {
        const bf16x8_t v = read_transposed(tile, ls, 32 * kk, (wave * OT + i) * 16, i16, g);
        o[i] = mfma_bf16(v, pf[kk][0], o[i]);
        o[i] = mfma_bf16(v, pf[kk][1], o[i]);
      }
    __syncthreads();
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (g == 0) wmax[wave * 16 + i16] = l;
  __syncthreads();
  l = (wmax[i16] + wmax[16 + i16]) + (wmax[32 + i16] + wmax[48 + i16]);
  if (head >= p.heads) return;
  const int64_t part = (t * p.heads + head) * p.splits + split;
  const float inv = p.splits == 1 ? inverse_sum(m / kLog2e, l, p.sinks, head) : 1.0f;
#pragma unroll
  for (int i = 0; i < OT; ++i) {
    const int c = (wave * OT + i) * 16 + 4 * g;
    if (c < p.rank) {                                          // (the rank is a multiple of 8 here)
      const float v[4] = {o[i][0] * inv, o[i][1] * inv, o[i][2] * inv, o[i][3] * inv};
      if (p.splits == 1) st4(static_cast<uint16_t*>(p.out) + t * p.o_token + head * p.o_head + c, v);
      else st4(p.part_o + part * p.rank + c, v);
    }
  }
  if (p.splits > 1 && wave == 0 && g == 0) {
    p.part_ml[part * 2] = m / kLog2e;
    p.part_ml[part * 2 + 1] = l;
  }
}

// ---------------------------------------------------------------------------------------------------------------
// Prefill: keys and values of the visible tokens expanded per head by one library product over the gathered latents, then
// flash attention.  A workgroup = 256 queries of one head (a wave = 32), key tiles of 64, the next tile's rows in registers while
// this one is multiplied; S^T = K Q^T leaves the weights of a query in the lane that needs them for O^T = V^T P^T, so they never touch LDS.
struct LatentPrefillParams {
  const void* q;             // [tokens, heads, dim + rot]
  int64_t q_token;
  const void* lat;           // [keys, row]: rotated parts at [rank, rank + rot)
  int64_t lat_stride;
  const void* kv;            // [keys, heads * dim | heads * vdim]
  int64_t kv_stride;
  const int32_t* blocks;     // [blocks, 2]: segment, first query within it
  const int32_t *seg_start, *seg_len, *key_start, *key_first;
  const int64_t* positions;
  void* out;                 // [tokens, heads * vdim]
  int64_t o_token;
  int heads, dim, rot, rank, vdim, window;
  float scale;
  const float* sinks;        // [heads], or null
};

constexpr int kPfThreads = 512;

template <int KS, int VT>
__global__ __launch_bounds__(kPfThreads, 2) void latent_prefill_kernel(LatentPrefillParams p) {
  constexpr int KLS = KS * 32 + 8, VLS = VT * 16 + 8;
  constexpr int KV8 = (kTile * KS * 4 + kPfThreads - 1) / kPfThreads, VV8 = (kTile * VT * 2 + kPfThreads - 1) / kPfThreads;
  __shared__ __attribute__((aligned(16))) uint16_t kimg[2][kTile * KLS];
  __shared__ __attribute__((aligned(16))) uint16_t vimg[2][kTile * VLS];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), i16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.x;
  const int b = p.blocks[2 * blockIdx.y], q0 = p.blocks[2 * blockIdx.y + 1];
  const int64_t t0 = p.seg_start[b];
  const int len = p.seg_len[b];
  const int pos0 = static_cast<int>(p.positions[t0]);
  const int64_t kbase = p.key_start[b];
  const int kfirst = p.key_first[b];
  const int q_last = q0 + 255 < len ? q0 + 255 : len - 1;
  int lo = pos0 + q0 - p.window + 1;
  if (p.window <= 0 || lo < kfirst) lo = kfirst;
  const int end = pos0 + q_last + 1;
  const int dk = p.dim + p.rot;

  bf16x8_t q[2][KS];
  int qpos[2];
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    int qi = q0 + 32 * wave + 16 * c + i16;
    if (qi >= len) qi = len - 1;
    qpos[c] = pos0 + qi;
    const uint16_t* qr = static_cast<const uint16_t*>(p.q) + (t0 + qi) * p.q_token + static_cast<int64_t>(h) * dk;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int e = 32 * k + 8 * g;
      U4 v = ld16(e < dk ? qr + e : qr);
      const uint32_t keep = e < dk ? 0xffffffffu : 0u;
      v.x &= keep; v.y &= keep; v.z &= keep; v.w &= keep;
      q[c][k] = as_frag(v);
    }
  }
  const int wave_first = pos0 + q0 + 32 * wave, wave_last = wave_first + 31;
  const uint16_t* kv = static_cast<const uint16_t*>(p.kv);
  const uint16_t* lat = static_cast<const uint16_t*>(p.lat);
  U4 kreg[KV8], vreg[VV8];
  // (addresses are clamped, never predicated: all loads stay in flight; what they should not have read is zeroed at the store)
  auto load = [&](int j0) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < KV8; ++i) {
      const int idx = i * kPfThreads + threadIdx.x, e = (idx % (KS * 4)) * 8;
      int j = j0 + idx / (KS * 4);
      j = j < end ? j : end - 1;
      const int64_t key = kbase + (j - kfirst);
      const uint16_t* kp = kv + key * p.kv_stride + h * p.dim + e;
      const uint16_t* rp = lat + key * p.lat_stride + p.rank + (e < dk ? e - p.dim : 0);
      kreg[i] = ld16(e < p.dim ? kp : rp);
    }
#pragma unroll
    for (int i = 0; i < VV8; ++i) {
      const int idx = i * kPfThreads + threadIdx.x, e = (idx % (VT * 2)) * 8;
      int j = j0 + idx / (VT * 2);
      j = j < end ? j : end - 1;
      vreg[i] = ld16(kv + (kbase + (j - kfirst)) * p.kv_stride + p.heads * p.dim + h * p.vdim + (e < p.vdim ? e : 0));
    }
  };
  f32x4_t o[2][VT];
  float m[2] = {-INFINITY, -INFINITY}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int c = 0; c < 2; ++c)
#pragma unroll
    for (int n = 0; n < VT; ++n) o[c][n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  const float sc = p.scale * kLog2e;
  load(lo);
  int image = 0;
  for (int j0 = lo; j0 < end; j0 += kTile, image ^= 1) {
    // (the barrier of the tile before this one lies behind every read of this image)
    uint16_t *kt = kimg[image], *vt = vimg[image];
#pragma unroll
    for (int i = 0; i < KV8; ++i) {
      const int idx = i * kPfThreads + threadIdx.x;
      const int r = idx / (KS * 4), e = (idx % (KS * 4)) * 8;
      if (r < kTile) st16(kt + r * KLS + e, keep_if(kreg[i], j0 + r < end && e < dk));
    }
#pragma unroll
    for (int i = 0; i < VV8; ++i) {
      const int idx = i * kPfThreads + threadIdx.x;
      const int r = idx / (VT * 2), e = (idx % (VT * 2)) * 8;
      if (r < kTile) st16(vt + r * VLS + e, keep_if(vreg[i], j0 + r < end && e < p.vdim));
    }
    __syncthreads();
    if (j0 + kTile < end) load(j0 + kTile);
    // a wave leaves out tiles none of its queries sees
    const bool seen = j0 <= wave_last && (p.window <= 0 || j0 + kTile - 1 > wave_first - p.window);
    if (seen) {
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
      const bool edge = j0 + kTile - 1 > wave_first || (p.window > 0 && j0 <= wave_last - p.window);
      bf16x8_t pf[2][2][2];
#pragma unroll
      for (int c = 0; c < 2; ++c) {
        // (the scale is positive: the largest product is the largest score)
        float mx = -INFINITY;
#pragma unroll
        for (int n = 0; n < 4; ++n)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            if (edge) {
              const int j = j0 + 16 * n + 4 * g + r;
              if (j > qpos[c] || (p.window > 0 && j <= qpos[c] - p.window)) s[c][n][r] = -INFINITY;
            }
            mx = fmaxf(mx, s[c][n][r]);
          }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float mn = fmaxf(m[c], mx * sc);
        const float base = mn == -INFINITY ? 0.f : mn;       // nothing visible yet: all weights zero
        float sum = 0.f;
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
          uint32_t wh[4], wl[4];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float e0 = fast_exp2(s[c][2 * kk + (j >> 1)][2 * (j & 1)] * sc - base);
            const float e1 = fast_exp2(s[c][2 * kk + (j >> 1)][2 * (j & 1) + 1] * sc - base);
            sum += e0 + e1;
            wh[j] = pack_bf2(e0, e1);
            wl[j] = pack_bf2(e0 - bf_lo(wh[j]), e1 - bf_hi(wh[j]));
          }
          pf[c][kk][0] = as_frag(U4{wh[0], wh[1], wh[2], wh[3]});
          pf[c][kk][1] = as_frag(U4{wl[0], wl[1], wl[2], wl[3]});
        }
        if (__any(mn != m[c])) {                               // some query's maximum moved
          const float fix = fast_exp2(m[c] - base);
          l[c] *= fix;
#pragma unroll
          for (int n = 0; n < VT; ++n) o[c][n] *= fix;
        }
        l[c] += sum;
        m[c] = mn;
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
  }
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    float sum = l[c];
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    const float inv = inverse_sum(m[c] / kLog2e, sum, p.sinks, h);
    const int qi = q0 + 32 * wave + 16 * c + i16;
    if (qi >= len) continue;
    uint16_t* orow = static_cast<uint16_t*>(p.out) + (t0 + qi) * p.o_token + static_cast<int64_t>(h) * p.vdim;
#pragma unroll
    for (int n = 0; n < VT; ++n) {
      const int e = 16 * n + 4 * g;
      if (e < p.vdim) {
        const float v[4] = {o[c][n][0] * inv, o[c][n][1] * inv, o[c][n][2] * inv, o[c][n][3] * inv};
        st4(orow + e, v);
      }
    }
  }
}

// rows of the visible keys, packed segment by segment
__global__ __launch_bounds__(256) void latent_gather_kernel(const uint16_t* __restrict__ cache, int64_t cache_stride, int vecs,
                                                            const int32_t* __restrict__ req_to_token, int64_t r2t_stride,
                                                            const int64_t* __restrict__ req, const int32_t* __restrict__ key_seg,
                                                            const int32_t* __restrict__ key_start, const int32_t* __restrict__ key_first,
                                                            uint16_t* __restrict__ out, int64_t out_stride, int64_t keys) {
  const int64_t i = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  const int64_t key = i / vecs;
  if (key >= keys) return;
  const int c = static_cast<int>(i - key * vecs) * 8;
  const int b = key_seg[key];
  const int64_t slot = req_to_token[req[b] * r2t_stride + key_first[b] + (key - key_start[b])];
  st16(out + key * out_stride + c, ld16(cache + slot * cache_stride + c));
}

template <int KS, int OT, int HG>
int launch_latent_mfma_hg(const LatentAttnParams& p, int64_t tokens, hipStream_t st) {
  const size_t lds = (static_cast<size_t>(kTile) * (KS * 32 + 8) + HG * 2 * 16 * (kTile + 8)) * 2 + HG * 64 * 4;
  if (lds > 64 * 1024) {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&latent_attention_mfma_kernel<KS, OT, HG>),
                                       hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds));
    SGL_CHECK_ARG(e == hipSuccess, "latent_attention: %zu bytes of LDS: %s", lds, hipGetErrorString(e));
  }
  hipLaunchKernelGGL((latent_attention_mfma_kernel<KS, OT, HG>), dim3(static_cast<unsigned>(tokens), (p.heads + 16 * HG - 1) / (16 * HG), p.splits),
                     dim3(256 * HG), lds, st, p);
  return 0;
}

template <int KS, int OT>
int launch_latent_mfma(const LatentAttnParams& p, int64_t tokens, hipStream_t st) {
  return p.heads > 16 ? launch_latent_mfma_hg<KS, OT, 2>(p, tokens, st) : launch_latent_mfma_hg<KS, OT, 1>(p, tokens, st);
}

}  // namespace

extern "C" {

int sgl_amd_latent_prepare(int is_f32, void* q, int64_t q_stride, const void* dkv, int64_t dkv_stride, const float* norm_weight,
                           const float* cos_sin, int64_t max_positions, const int64_t* positions, const int64_t* loc, void* cache,
                           int64_t cache_stride, int64_t tokens, int heads, int dim, int rot, int rot_dims, int rank, float eps, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(q && dkv && norm_weight && cos_sin && positions && loc && cache, "latent_prepare: null operand");
  SGL_CHECK_ARG(rot_dims % 2 == 0 && rot_dims <= rot && rank > 0 && heads > 0 && dim >= 0 && cache_stride >= rank + rot && max_positions > 0,
                "latent_prepare: rank %d, rot %d (%d rotated), row %lld", rank, rot, rot_dims, (long long)cache_stride);
  if (tokens <= 0) return 0;
  PrepareParams p{q, q_stride, dkv, dkv_stride, norm_weight, cos_sin, positions, loc, cache, cache_stride,
                  heads, dim, rot, rot_dims, rank, max_positions, eps, 0};
  const size_t al = is_f32 ? 16 : 8;
  p.vec = rank % 4 == 0 && dim % 4 == 0 && rot % 4 == 0 && rot_dims == rot && q_stride % 4 == 0 && dkv_stride % 4 == 0 && cache_stride % 4 == 0 &&
          aligned_to(q, al) && aligned_to(dkv, al) && aligned_to(cache, al) && aligned_to(norm_weight, 16);
  if (is_f32) hipLaunchKernelGGL((latent_prepare_kernel<float>), dim3(static_cast<unsigned>(tokens)), dim3(256), 0, as_stream(stream), p);
  else hipLaunchKernelGGL((latent_prepare_kernel<uint16_t>), dim3(static_cast<unsigned>(tokens)), dim3(256), 0, as_stream(stream), p);
  SGL_CHECK_LAUNCH("latent_prepare");
  return 0;
}

int sgl_amd_head_gemm(int is_f32, const void* x, int64_t x_token_stride, int64_t x_head_stride, const void* w, void* out,
                      int64_t o_token_stride, int64_t o_head_stride, int64_t tokens, int heads, int N, int K, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(x && w && out && heads > 0 && heads <= 65535 && N > 0 && K > 0, "head_gemm: %d heads, %d x %d", heads, N, K);
  if (tokens <= 0) return 0;
  HeadGemmParams p{x, x_token_stride, x_head_stride, w, out, o_token_stride, o_head_stride, tokens, N, K,
                   o_token_stride % 4 == 0 && o_head_stride % 4 == 0 && aligned_to(out, 8) ? 1 : 0};
  hipStream_t st = as_stream(stream);
  const bool mfma = !is_f32 && K % 8 == 0 && x_token_stride % 8 == 0 && x_head_stride % 8 == 0 && aligned_to(x, 16) && aligned_to(w, 16) &&
                    (tokens + 15) / 16 <= 65535;
  if (mfma) {
    const unsigned nb = (N + 15) / 16;
    if (tokens <= 16) hipLaunchKernelGGL((head_gemm_mfma_kernel<1>), dim3(nb, heads, 1), dim3(256), 0, st, p);
    else if (tokens <= 32) hipLaunchKernelGGL((head_gemm_mfma_kernel<2>), dim3(nb, heads, 1), dim3(256), 0, st, p);
    else hipLaunchKernelGGL((head_gemm_mfma_kernel<4>), dim3(nb, heads, static_cast<unsigned>((tokens + 63) / 64)), dim3(256), 0, st, p);
  } else {
    const dim3 grid(static_cast<unsigned>(tokens), heads, (N + 255) / 256);
    if (is_f32) hipLaunchKernelGGL((head_gemm_plain_kernel<float>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((head_gemm_plain_kernel<uint16_t>), grid, dim3(256), 0, st, p);
  }
  SGL_CHECK_LAUNCH("head_gemm");
  return 0;
}

int sgl_amd_latent_attention(int is_f32, const void* qc, int64_t qc_token, int64_t qc_head, const void* qr, int64_t qr_token,
                             int64_t qr_head, const void* cache, int64_t cache_stride, const int32_t* req_to_token, int64_t r2t_stride,
                             const int64_t* req_pool_indices, const int32_t* tok_seg, const int64_t* positions, void* out, int64_t o_token,
                             int64_t o_head, float* part_o, float* part_ml, int64_t tokens, int heads, int rank, int rot, int window,
                             int splits, float scale, const float* sinks, int plain, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(qc && qr && cache && req_to_token && req_pool_indices && positions && out, "latent_attention: null operand");
  SGL_CHECK_ARG(heads > 0 && heads <= 65535 && rank > 0 && rot >= 0 && cache_stride >= rank + rot && splits >= 1 && splits <= 64,
                "latent_attention: %d heads, rank %d, rot %d, %d splits", heads, rank, rot, splits);
  SGL_CHECK_ARG(splits == 1 || (part_o && part_ml), "latent_attention: split launches need their workspaces");
  if (tokens <= 0) return 0;
  LatentAttnParams p{qc, qc_token, qc_head, qr, qr_token, qr_head, cache, cache_stride, req_to_token, r2t_stride, req_pool_indices, tok_seg,
                     positions, out, o_token, o_head, part_o, part_ml, heads, rank, rot, window, splits, scale, sinks};
  // queries in whole 16-byte pieces
  const bool vecq = rank % 8 == 0 && rot % 8 == 0 && qc_token % 8 == 0 && qc_head % 8 == 0 && qr_token % 8 == 0 && qr_head % 8 == 0 &&
           aligned_to(qc, 16) && aligned_to(qr, 16) && o_token % 4 == 0 && o_head % 4 == 0 && aligned_to(out, 8) && aligned_to(part_o, 16);
  hipStream_t st = as_stream(stream);
  const int dk = (rank + rot + 31) / 32 * 32;
  if (!is_f32 && !plain && vecq && rank <= 512 && dk <= 640 && cache_stride % 8 == 0 && cache_stride >= dk && aligned_to(cache, 16)) {
    const int rc = rank <= 64 && dk <= 128    ? launch_latent_mfma<4, 1>(p, tokens, st)
                   : rank <= 128 && dk <= 256 ? launch_latent_mfma<8, 2>(p, tokens, st)
                   : rank <= 256 && dk <= 384 ? launch_latent_mfma<12, 4>(p, tokens, st)
                   : dk <= 576                ? launch_latent_mfma<18, 8>(p, tokens, st)
                                              : launch_latent_mfma<20, 8>(p, tokens, st);
    if (rc) return rc;
    if (splits > 1) launch_latent_merge<uint16_t>(p, tokens, st);
    SGL_CHECK_LAUNCH("latent_attention");
    return 0;
  }
  const dim3 grid(static_cast<unsigned>(tokens), heads, splits);
  const size_t lds = (2 * static_cast<size_t>(rank) + rot + 512) * 4;
  SGL_CHECK_ARG(lds <= 64 * 1024 - 256, "latent_attention: rank %d needs %zu bytes of LDS", rank, lds);
  if (is_f32) hipLaunchKernelGGL((latent_attention_plain_kernel<float>), grid, dim3(256), lds, st, p);
  else hipLaunchKernelGGL((latent_attention_plain_kernel<uint16_t>), grid, dim3(256), lds, st, p);
  if (splits > 1) {
    if (is_f32) launch_latent_merge<float>(p, tokens, st);
    else launch_latent_merge<uint16_t>(p, tokens, st);
  }
  SGL_CHECK_LAUNCH("latent_attention");
  return 0;
}

int sgl_amd_latent_prefill_supported(int dim, int rot, int vdim) {
  return dim % 8 == 0 && rot >= 8 && rot % 8 == 0 && vdim % 8 == 0 && dim + rot <= 256 && vdim <= 128 ? 1 : 0;
}

int sgl_amd_latent_gather(const void* cache, int64_t cache_stride, const int32_t* req_to_token, int64_t r2t_stride,
                          const int64_t* req_pool_indices, const int32_t* key_seg, const int32_t* key_start, const int32_t* key_first,
                          void* out, int64_t out_stride, int64_t keys, int row, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(cache && req_to_token && req_pool_indices && key_seg && key_start && key_first && out, "latent_gather: null operand");
  SGL_CHECK_ARG(row > 0 && row % 8 == 0 && cache_stride % 8 == 0 && out_stride % 8 == 0 && aligned_to(cache, 16) && aligned_to(out, 16),
                "latent_gather: rows of whole 16-byte vectors");
  if (keys <= 0) return 0;
  const int vecs = row / 8;
  hipLaunchKernelGGL(latent_gather_kernel, dim3(static_cast<unsigned>((keys * vecs + 255) / 256)), dim3(256), 0, as_stream(stream),
                     static_cast<const uint16_t*>(cache), cache_stride, vecs, req_to_token, r2t_stride, req_pool_indices, key_seg, key_start,
                     key_first, static_cast<uint16_t*>(out), out_stride, keys);
  SGL_CHECK_LAUNCH("latent_gather");
  return 0;
}

int sgl_amd_latent_prefill(const void* q, int64_t q_token, const void* latents, int64_t latents_stride, const void* kv, int64_t kv_stride,
                           const int32_t* blocks, int num_blocks, const int32_t* seg_start, const int32_t* seg_len, const int32_t* key_start,
                           const int32_t* key_first, const int64_t* positions, void* out, int64_t o_token, int heads, int dim, int rot,
                           int rank, int vdim, int window, float scale, const float* sinks, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  SGL_CHECK_ARG(q && latents && kv && blocks && seg_start && seg_len && key_start && key_first && positions && out, "latent_prefill: null operand");
  SGL_CHECK_ARG(sgl_amd_latent_prefill_supported(dim, rot, vdim) && heads > 0 && rank % 8 == 0 && num_blocks <= 65535,
                "latent_prefill: dims %d + %d, value %d, rank %d", dim, rot, vdim, rank);
  SGL_CHECK_ARG(scale > 0.f, "latent_prefill: the scale must be positive");
  SGL_CHECK_ARG(q_token % 8 == 0 && latents_stride % 8 == 0 && kv_stride % 8 == 0 && o_token % 4 == 0 && aligned_to(q, 16) && aligned_to(latents, 16) &&
                    aligned_to(kv, 16) && aligned_to(out, 8),
                "latent_prefill: rows of whole 16-byte vectors");
  if (num_blocks <= 0) return 0;
  LatentPrefillParams p{q, q_token, latents, latents_stride, kv, kv_stride, blocks, seg_start, seg_len, key_start, key_first, positions, out, o_token,
                        heads, dim, rot, rank, vdim, window, scale, sinks};
  const dim3 grid(heads, num_blocks);
  hipStream_t st = as_stream(stream);
  const int dk = dim + rot;
  if (dk <= 128 && vdim <= 64) hipLaunchKernelGGL((latent_prefill_kernel<4, 4>), grid, dim3(kPfThreads), 0, st, p);
  else if (dk <= 192 && vdim <= 128) hipLaunchKernelGGL((latent_prefill_kernel<6, 8>), grid, dim3(kPfThreads), 0, st, p);
  else hipLaunchKernelGGL((latent_prefill_kernel<8, 8>), grid, dim3(kPfThreads), 0, st, p);
  SGL_CHECK_LAUNCH("latent_prefill");
  return 0;
}

}  // extern "C"
