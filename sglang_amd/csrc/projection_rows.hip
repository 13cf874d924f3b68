// What stands between a projection and attention, one launch each: split-K sums and biases, norms, rotation by halves, the cache rows.
//
//   head_prepare   rows [query heads | key heads | value heads | gate]: an RMS norm a head in front of the rotation (with weights) or behind
//                  it (without), rotation of dimension i with i + dims / 2; queries to their rows, keys and values to the cache.  Where a
//                  design's values are its keys, there are no value columns: they are the key columns as projected
//   latent_down    rows [query latent | latent | rotated key part]: RMS norms of both latents, rotation of the key part, the cache row
//
// Sources are rows in the activation type or the fp32 split-K partials of a decode projection; everything up to the store is fp32.
#include "elem_io.hpp"
#include "sglang_amd.h"

using namespace sgl_amd;

namespace {

// row t of a projection: rows at `stride`, or `items` partials `item_stride` apart plus a bias
struct ProjRows {
  const void* rows;
  int64_t stride;
  const float* part;
  int items;
  int64_t item_stride;
  const void* bias;          // [columns] activation type, partials only; or null
};

template <typename T, int VEC>
__device__ __forceinline__ void load_projection(const ProjRows& s, int64_t t, int64_t c, float (&v)[VEC]) {
  if (!s.part) {
    ldv<VEC>(static_cast<const T*>(s.rows) + t * s.stride + c, v);
    return;
  }
  const float* p = s.part + t * s.stride + c;
#pragma unroll
  for (int j = 0; j < VEC; ++j) v[j] = 0.f;
  for (int i = 0; i < s.items; i += 4) {               // four loads in flight, clamped to the last item
    float u[4][VEC];
#pragma unroll
    for (int q = 0; q < 4; ++q) ldv<VEC>(p + static_cast<int64_t>(i + q < s.items ? i + q : s.items - 1) * s.item_stride, u[q]);
#pragma unroll
    for (int q = 0; q < 4; ++q)
      if (i + q < s.items) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += u[q][j];
      }
  }
  if (s.bias) {
    float b[VEC];
    ldv<VEC>(static_cast<const T*>(s.bias) + c, b);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] += b[j];
  }
}

struct HeadPrepareParams {
  ProjRows src;
  void* out;                 // [tokens, heads * kd (| gate columns of partials)]; may be the source's rows
  int64_t o_stride;
  const float *q_norm, *k_norm;      // [kd], order 1
  const float* cos_sin;      // [positions, rot_dims]: cos | sin, or null
  int64_t max_pos;
  const int64_t* positions;
  void* cache;               // rows [kv_heads][kd | vd]
  int64_t cache_stride;
  const int64_t* loc;
  int64_t tokens;
  int heads, kv_heads, kd, vd, dim, rot_off, rot_dims, norm_order, gate_cols, units, in_place;
  int value_is_key;          // the values are the keys in front of norm and rotation (vd == kd)
  int q_off, q_width;        // the columns of a query head this launch touches
  float eps;
};

struct HeadUnit {
  int kind, width;           // 0 query, 1 key, 2 value, 3 gate
  int64_t col, dst;          // first source column; first element of out's row or of the cache row
};

__device__ __forceinline__ HeadUnit head_unit(const HeadPrepareParams& p, int u, int gate_piece) {
  const int H = p.heads, G = p.kv_heads;
  if (u < H) return {0, p.q_width, static_cast<int64_t>(u) * p.kd + p.q_off, static_cast<int64_t>(u) * p.kd + p.q_off};
  const int64_t k0 = static_cast<int64_t>(H) * p.kd, k1 = k0 + static_cast<int64_t>(G) * p.kd;
  const int64_t v0 = p.value_is_key ? k0 : k1, g0 = p.value_is_key ? k1 : k1 + static_cast<int64_t>(G) * p.vd;
  u -= H;
  if (u < G) return {1, p.kd, k0 + static_cast<int64_t>(u) * p.kd, static_cast<int64_t>(u) * (p.kd + p.vd)};
  u -= G;
  if (u < G) return {2, p.vd, v0 + static_cast<int64_t>(u) * p.vd, static_cast<int64_t>(u) * (p.kd + p.vd) + p.kd};
  u -= G;
  const int left = p.gate_cols - u * gate_piece;
  return {3, left < gate_piece ? left : gate_piece, g0 + static_cast<int64_t>(u) * gate_piece, k0 + static_cast<int64_t>(u) * gate_piece};
}

template <typename T>
__device__ __forceinline__ T* unit_dst(const HeadPrepareParams& p, const HeadUnit& u, int64_t t) {
  return u.kind == 0 || u.kind == 3 ? static_cast<T*>(p.out) + t * p.o_stride + u.dst : static_cast<T*>(p.cache) + p.loc[t] * p.cache_stride + u.dst;
}

__device__ __forceinline__ const float* rotation(const HeadPrepareParams& p, int64_t t) {
  int64_t pos = p.positions[t];
  if (pos >= p.max_pos) pos = p.max_pos - 1;           // (the host never passes one)
  return p.cos_sin + pos * p.rot_dims;
}

// TPH lanes a head, eight columns a lane; halves of whole pieces, so a rotation partner is another lane's piece.
template <typename T, int TPH>
__global__ __launch_bounds__(256) void head_prepare_kernel(HeadPrepareParams p) {
  const int64_t item = static_cast<int64_t>(blockIdx.x) * (256 / TPH) + threadIdx.x / TPH;
  const bool live = item < p.tokens * p.units;
  const int64_t t = live ? item / p.units : 0;
  const HeadUnit u = head_unit(p, live ? static_cast<int>(item - t * p.units) : 0, TPH * 8);
  const int lane = threadIdx.x & 63, c = static_cast<int>(threadIdx.x % TPH) * 8;
  const int half = p.rot_dims >> 1, r = c - p.rot_off;
  const bool head = u.kind < 2, turns = head && p.cos_sin && r >= 0 && r < p.rot_dims;
  const bool active = live && c < u.width;
  float v[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = 0.f;
  if (active) load_projection<T, 8>(p.src, t, u.col + c, v);
  auto unit_scale = [&]() __attribute__((always_inline)) {
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) ss += v[j] * v[j];
#pragma unroll
    for (int off = TPH / 2; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
    return 1.0f / sqrtf(ss / static_cast<float>(p.dim) + p.eps);
  };
  if (p.norm_order == 1) {
    const float rs = unit_scale();
    if (head) {
      const float* w = u.kind == 0 ? p.q_norm : p.k_norm;
      float wv[8];
      ldv<8>(w + (active ? c : 0), wv);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] *= rs * wv[j];
    }
  }
  if (p.cos_sin) {
    const bool first = r < half;
    const int from = turns ? lane + (first ? half : -half) / 8 : lane;
    float o[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = __shfl(v[j], from, 64);
    if (turns && active) {
      const float* cs = rotation(p, t) + (first ? r : r - half);
      float co[8], si[8];
      ldv<8>(cs, co);
      ldv<8>(cs + half, si);
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] = first ? v[j] * co[j] - o[j] * si[j] : v[j] * co[j] + o[j] * si[j];
    }
  }
  if (p.norm_order == 2) {
    const float rs = unit_scale();
    if (head) {
#pragma unroll
      for (int j = 0; j < 8; ++j) v[j] *= rs;
    }
  }
  if (active) stv<8>(unit_dst<T>(p, u, t) + c, v);
}

// Any sizes: a wave per (token, head), the head in LDS.
template <typename T>
__global__ __launch_bounds__(256) void head_prepare_plain_kernel(HeadPrepareParams p, int row) {
  extern __shared__ float lds[];
  const int lane = threadIdx.x & 63;
  const int64_t item = static_cast<int64_t>(blockIdx.x) * 4 + (threadIdx.x >> 6);
  if (item >= p.tokens * p.units) return;
  float* x = lds + (threadIdx.x >> 6) * row;
  const int64_t t = item / p.units;
  const HeadUnit u = head_unit(p, static_cast<int>(item - t * p.units), row);
  T* dst = unit_dst<T>(p, u, t);
  float ss = 0.f;
  for (int c = lane; c < u.width; c += 64) {
    float v[1];
    load_projection<T, 1>(p.src, t, u.col + c, v);
    x[c] = v[0];
    ss += v[0] * v[0];
  }
  asm volatile("" ::: "memory");                       // (a wave's own row: LDS serves a wave in order)
  __builtin_amdgcn_wave_barrier();
  const bool head = u.kind < 2;
  const float before = 1.0f / sqrtf(wave_sum(ss) / static_cast<float>(p.dim) + p.eps);
  const float* w = u.kind == 0 ? p.q_norm : p.k_norm;
  const float* cs = p.cos_sin && head ? rotation(p, t) : nullptr;
  const int half = p.rot_dims >> 1;
  auto at = [&](int c) { return head && p.norm_order == 1 ? x[c] * before * w[c] : x[c]; };
  auto turned = [&](int c) {
    const int r = c - p.rot_off;
    if (!cs || r < 0 || r >= p.rot_dims) return at(c);
    return r < half ? at(c) * cs[r] - at(c + half) * cs[half + r] : at(c) * cs[r - half] + at(c - half) * cs[r];
  };
  float after = 1.0f;
  if (head && p.norm_order == 2) {
    float sq = 0.f;
    for (int c = lane; c < u.width; c += 64) { const float v = turned(c); sq += v * v; }
    after = 1.0f / sqrtf(wave_sum(sq) / static_cast<float>(p.dim) + p.eps);
  }
  for (int c = lane; c < u.width; c += 64) st1(dst + c, turned(c) * after);
}

// ---------------------------------------------------------------------------------------------------------------
struct LatentDownParams {
  ProjRows src;              // [tokens, q_rank + rank + rot]
  const float *q_norm, *norm;        // [q_rank], [rank]
  const float* cos_sin;      // [positions, rot_dims]
  int64_t max_pos;
  const int64_t *positions, *loc;
  void* cq;                  // [tokens, q_rank]
  int64_t cq_stride;
  void* cache;               // rows [rank | rot]
  int64_t cache_stride;
  int q_rank, rank, rot, rot_dims;
  float eps;
};

template <typename T, int VEC>
__global__ __launch_bounds__(256) void latent_down_kernel(LatentDownParams p) {
  extern __shared__ float x[];
  __shared__ float scratch[16];
  const int64_t t = blockIdx.x;
  const int n = p.q_rank + p.rank + p.rot, latent = p.q_rank + p.rank;
  float sq = 0.f, sc = 0.f;
  for (int c = threadIdx.x * VEC; c < n; c += 256 * VEC) {
    float v[VEC];
    load_projection<T, VEC>(p.src, t, c, v);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      x[c + j] = v[j];
      if (c < p.q_rank) sq += v[j] * v[j];
      else if (c < latent) sc += v[j] * v[j];
    }
  }
  sq = block_sum(sq, scratch);
  sc = block_sum(sc, scratch);
  const float rq = p.q_rank ? 1.0f / sqrtf(sq / static_cast<float>(p.q_rank) + p.eps) : 0.f;
  const float rc = 1.0f / sqrtf(sc / static_cast<float>(p.rank) + p.eps);
  T* cq = static_cast<T*>(p.cq) + t * p.cq_stride;
  T* row = static_cast<T*>(p.cache) + p.loc[t] * p.cache_stride;
  for (int c = threadIdx.x * VEC; c < latent; c += 256 * VEC) {
    const bool q = c < p.q_rank;
    const int e = q ? c : c - p.q_rank;
    const float f = q ? rq : rc;
    float w[VEC], o[VEC];
    ldv<VEC>((q ? p.q_norm : p.norm) + e, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = x[c + j] * f * w[j];
    stv<VEC>((q ? cq : row) + e, o);
  }
  int64_t pos = p.positions[t];
  if (pos >= p.max_pos) pos = p.max_pos - 1;           // (the host never passes one)
  const float* cs = p.cos_sin + pos * p.rot_dims;
  const int half = p.rot_dims >> 1;
  const float* k = x + latent;
  for (int r = threadIdx.x; r < p.rot; r += 256) {
    float v = k[r];
    if (r < half) v = v * cs[r] - k[r + half] * cs[half + r];
    else if (r < p.rot_dims) v = v * cs[r - half] + k[r - half] * cs[r];
    st1(row + p.rank + r, v);
  }
}

bool source_ok(const ProjRows& s) { return s.part ? s.items >= 1 : s.rows != nullptr; }
bool source_vec(const ProjRows& s, int vec, size_t bytes) {
  return s.part ? s.stride % vec == 0 && s.item_stride % vec == 0 && aligned_to(s.part, 16) && aligned_to(s.bias, bytes)
                : s.stride % vec == 0 && aligned_to(s.rows, bytes);
}

template <typename T>
void launch_head_prepare(const HeadPrepareParams& p0, bool vec, hipStream_t st) {
  HeadPrepareParams p = p0;
  p.q_off = 0; p.q_width = p.kd;
  if (p.in_place && !p.norm_order && !p.kv_heads && !p.gate_cols) {            // nothing but the turned columns changes
    if (!p.rot_dims) return;
    p.q_off = p.rot_off; p.q_width = p.rot_dims; p.rot_off = 0;
  }
  const int widest = p.kv_heads && p.vd > p.q_width ? p.vd : p.q_width, plain_units = p.heads + 2 * p.kv_heads;
  if (vec && widest <= 512) {
    const int tph = widest <= 64 ? 8 : widest <= 128 ? 16 : widest <= 256 ? 32 : 64;
    p.units = plain_units + (p.gate_cols + tph * 8 - 1) / (tph * 8);
    const dim3 grid(static_cast<unsigned>((p.tokens * p.units * tph + 255) / 256));
    if (tph == 8) hipLaunchKernelGGL((head_prepare_kernel<T, 8>), grid, dim3(256), 0, st, p);
    else if (tph == 16) hipLaunchKernelGGL((head_prepare_kernel<T, 16>), grid, dim3(256), 0, st, p);
    else if (tph == 32) hipLaunchKernelGGL((head_prepare_kernel<T, 32>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((head_prepare_kernel<T, 64>), grid, dim3(256), 0, st, p);
  } else {
    p.units = plain_units + (p.gate_cols + widest - 1) / widest;
    const dim3 grid(static_cast<unsigned>((p.tokens * p.units + 3) / 4));
    hipLaunchKernelGGL((head_prepare_plain_kernel<T>), grid, dim3(256), static_cast<size_t>(widest) * 16, st, p, widest);
  }
}

}  // namespace

extern "C" {

int sgl_amd_head_prepare(int is_f32, const void* rows, int64_t row_stride, const float* partials, int items, int64_t item_stride, const void* bias,
                         void* out, int64_t o_stride, const float* q_norm, const float* k_norm, int norm_order, float eps, const float* cos_sin,
                         int64_t max_positions, const int64_t* positions, int rot_off, int rot_dims, void* cache, int64_t cache_stride,
                         const int64_t* loc, int64_t tokens, int heads, int kv_heads, int kd, int vd, int dim, int gate_cols, int value_is_key, int plain,
                         void* stream) {
  SGL_CLEAR_STALE_ERROR();
  HeadPrepareParams p{};
  p.src = ProjRows{rows, row_stride, partials, items, item_stride, bias};
  SGL_CHECK_ARG(source_ok(p.src) && out && heads > 0 && kv_heads >= 0 && kd > 0 && dim > 0 && dim <= kd && (!kv_heads || (vd > 0 && cache && loc)),
                "head_prepare: %d / %d heads of %d (%d) + %d", heads, kv_heads, kd, dim, vd);
  SGL_CHECK_ARG(norm_order >= 0 && norm_order <= 2 && (norm_order != 1 || (q_norm && (!kv_heads || k_norm))), "head_prepare: norm %d without its weights", norm_order);
  SGL_CHECK_ARG(!cos_sin || (positions && max_positions > 0 && rot_dims > 0 && rot_dims % 2 == 0 && rot_off >= 0 && rot_off + rot_dims <= dim),
                "head_prepare: %d rotated dimensions from %d of %d", rot_dims, rot_off, dim);
  SGL_CHECK_ARG(kd <= 2048 && vd <= 2048 && cache_stride >= static_cast<int64_t>(kv_heads) * (kd + vd) && gate_cols >= 0 && tokens <= (1 << 24),
                "head_prepare: heads of %d + %d in rows of %lld", kd, vd, (long long)cache_stride);
  SGL_CHECK_ARG(!value_is_key || (kv_heads && vd == kd), "head_prepare: values of %d that are keys of %d", vd, kd);
  if (tokens <= 0) return 0;
  p.value_is_key = value_is_key;
  p.out = out; p.o_stride = o_stride; p.q_norm = q_norm; p.k_norm = k_norm; p.cos_sin = cos_sin; p.max_pos = max_positions; p.positions = positions;
  p.cache = cache; p.cache_stride = cache_stride; p.loc = loc; p.tokens = tokens; p.heads = heads; p.kv_heads = kv_heads; p.kd = kd; p.vd = vd;
  p.dim = dim; p.rot_off = rot_off; p.rot_dims = cos_sin ? rot_dims : 0; p.norm_order = norm_order; p.gate_cols = gate_cols;
  p.in_place = !partials && out == rows; p.eps = eps;
  SGL_CHECK_ARG(!p.in_place || o_stride == row_stride, "head_prepare: in place with another row stride");
  const bool vec = !plain && kd % 8 == 0 && (!kv_heads || vd % 8 == 0) && gate_cols % 8 == 0 && p.rot_dims % 16 == 0 && rot_off % 8 == 0 &&
                   source_vec(p.src, 8, 16) && o_stride % 8 == 0 && cache_stride % 8 == 0 && aligned_to(out, 16) && aligned_to(cache, 16) && aligned_to(cos_sin, 16) &&
                   aligned_to(q_norm, 16) && aligned_to(k_norm, 16);
  if (is_f32) launch_head_prepare<float>(p, vec, as_stream(stream));
  else launch_head_prepare<uint16_t>(p, vec, as_stream(stream));
  SGL_CHECK_LAUNCH("head_prepare");
  return 0;
}

int sgl_amd_latent_down(int is_f32, const void* rows, int64_t row_stride, const float* partials, int items, int64_t item_stride,
                        const float* q_norm, const float* norm, float eps, const float* cos_sin, int64_t max_positions, const int64_t* positions,
                        int rot_dims, void* cq, int64_t cq_stride, void* cache, int64_t cache_stride, const int64_t* loc, int64_t tokens,
                        int q_rank, int rank, int rot, void* stream) {
  SGL_CLEAR_STALE_ERROR();
  LatentDownParams p{ProjRows{rows, row_stride, partials, items, item_stride, nullptr}, q_norm, norm, cos_sin, max_positions, positions, loc,
                     cq, cq_stride, cache, cache_stride, q_rank, rank, rot, rot_dims, eps};
  SGL_CHECK_ARG(source_ok(p.src) && norm && cos_sin && positions && loc && cache && rank > 0 && q_rank >= 0 && (!q_rank || (cq && q_norm)) && rot >= 0 &&
                    rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= rot && cache_stride >= rank + rot && max_positions > 0,
                "latent_down: ranks %d and %d, %d rotated of %d, row %lld", q_rank, rank, rot_dims, rot, (long long)cache_stride);
  const size_t lds = (static_cast<size_t>(q_rank) + rank + rot) * 4;
  SGL_CHECK_ARG(lds <= 60 * 1024 && tokens <= 0x7fffffffLL, "latent_down: %zu bytes of LDS", lds);
  if (tokens <= 0) return 0;
  const size_t al = is_f32 ? 16 : 8;
  const bool vec = q_rank % 4 == 0 && rank % 4 == 0 && rot % 4 == 0 && source_vec(p.src, 4, al) && cq_stride % 4 == 0 && cache_stride % 4 == 0 &&
                   aligned_to(cq, al) && aligned_to(cache, al) && aligned_to(q_norm, 16) && aligned_to(norm, 16);
  const dim3 grid(static_cast<unsigned>(tokens));
  hipStream_t st = as_stream(stream);
  if (is_f32) {
    if (vec) hipLaunchKernelGGL((latent_down_kernel<float, 4>), grid, dim3(256), lds, st, p);
    else hipLaunchKernelGGL((latent_down_kernel<float, 1>), grid, dim3(256), lds, st, p);
  } else {
    if (vec) hipLaunchKernelGGL((latent_down_kernel<uint16_t, 4>), grid, dim3(256), lds, st, p);
    else hipLaunchKernelGGL((latent_down_kernel<uint16_t, 1>), grid, dim3(256), lds, st, p);
  }
  SGL_CHECK_LAUNCH("latent_down");
  return 0;
}

}  // extern "C"
