// Attention over latents: what a row's projections become before the product that makes its queries.
//
//   latent_rows   a row holds (each optional) the queries' latent of q_rank values, and the keys' latent of r values with n values behind it that are
//                 turned by the row's position and shared by all heads. The queries' latent is normed (RMS norm with a weight) into a buffer of its
//                 own. The keys' latent is normed likewise; with the turned values in front of it, [turned n | latent r | zeros], it goes to the row's
//                 cache slot as a key of d channels and, transposed, as a value whose first n channels are zero; or, where the pages do not hold
//                 latents, the normed latent and the n values as they are go side by side into rows of a buffer, zeros behind them.
//   turn_pairs    channels first + 2 i and first + 2 i + 1, i < pairs, of every head of a row turned in place by the row's position.
//
// Angles come from a table: cos, sin [positions, pairs], float32. Norms and turns are float arithmetic, double in the exact path.
#include "common.h"

namespace alofa {

struct LatentRows {
  int64_t x_stride;
  int q_at, q_rank;            // the queries' latent: its first column and its size (q_rank 0: none)
  const float* q_weight;
  float q_eps;
  int64_t cq_stride;
  int kv_at, r, n;             // the keys' latent: its first column and its size; the turned values lie right behind it
  const float* kv_weight;
  float kv_eps;
  const int32_t* positions;
  const float* cos_t;
  const float* sin_t;
  const int64_t* slots;        // pages
  int block_size, d;
  int64_t row_stride;          // rows: width of the room, zeros behind r + n
  int row_width;
};

// A block of four wavefronts per (row, latent): the keys' latents are the first `tokens` blocks, the queries' follow.
template <typename T, typename Acc>
__global__ void __launch_bounds__(256) latent_rows_kernel(const T* __restrict__ x, T* __restrict__ cq, T* __restrict__ k_cache, T* __restrict__ v_cache,
                                                          T* __restrict__ rows_out, int tokens, LatentRows a) {
  __shared__ Acc scratch[4];
  const bool of_keys = static_cast<int>(blockIdx.x) < tokens;
  const int t = of_keys ? blockIdx.x : blockIdx.x - tokens, tid = threadIdx.x;
  const T* src = x + static_cast<int64_t>(t) * a.x_stride + (of_keys ? a.kv_at : a.q_at);
  const int width = of_keys ? a.r : a.q_rank;
  const float* w = of_keys ? a.kv_weight : a.q_weight;
  // (what the stores below need is asked for with the row itself)
  int64_t slot = 0;
  const bool paged = of_keys && !rows_out;
  if (paged) slot = a.slots[t];
  const int64_t at = (paged && a.n > 0) ? static_cast<int64_t>(a.positions[t]) * (a.n / 2) : 0;
  constexpr int kOwn = 4;      // values a thread keeps (latents of up to 1,024 values; longer ones are read again)
  float own[kOwn], weight[kOwn];
  Acc ss = 0;
#pragma unroll
  for (int i = 0; i < kOwn; ++i) {
    const int c = tid + i * 256;
    own[i] = c < width ? load_f32(src + c) : 0.f;
    weight[i] = c < width ? w[c] : 0.f;
    ss += static_cast<Acc>(own[i]) * static_cast<Acc>(own[i]);
  }
  for (int c = tid + kOwn * 256; c < width; c += 256) ss += static_cast<Acc>(load_f32(src + c)) * static_cast<Acc>(load_f32(src + c));
  const Acc inv = static_cast<Acc>(1) / sqrt(block_sum<Acc, 256>(ss, scratch) / static_cast<Acc>(width) + static_cast<Acc>(of_keys ? a.kv_eps : a.q_eps));
  T *dst, *dst_v = nullptr;
  int64_t v_step = 0;
  int first = 0;
  if (!of_keys) {
    dst = cq + static_cast<int64_t>(t) * a.cq_stride;
  } else if (rows_out) {
    dst = rows_out + static_cast<int64_t>(t) * a.row_stride;
  } else {
    const int64_t page = slot / a.block_size, place = slot % a.block_size;
    dst = k_cache + (page * a.block_size + place) * a.d;
    dst_v = v_cache + page * a.d * a.block_size + place;
    v_step = a.block_size;
    first = a.n;
  }
  auto put = [&](float v, float wc, int c) {
    const float y = static_cast<float>(static_cast<Acc>(v) * inv * static_cast<Acc>(wc));
    store_f32(dst + first + c, y);
    if (dst_v) store_f32(dst_v + (first + c) * v_step, y);
  };
#pragma unroll
  for (int i = 0; i < kOwn; ++i)
    if (tid + i * 256 < width) put(own[i], weight[i], tid + i * 256);
  for (int c = tid + kOwn * 256; c < width; c += 256) put(load_f32(src + c), w[c], c);
  if (!of_keys) return;
  if (rows_out) {
    for (int c = tid; c < a.row_width - a.r; c += 256) store_f32(dst + a.r + c, c < a.n ? load_f32(src + a.r + c) : 0.f);
    return;
  }
  for (int i = tid; i < a.n / 2; i += 256) {
    const Acc u = static_cast<Acc>(load_f32(src + a.r + 2 * i)), v = static_cast<Acc>(load_f32(src + a.r + 2 * i + 1));
    const Acc cs = static_cast<Acc>(a.cos_t[at + i]), sn = static_cast<Acc>(a.sin_t[at + i]);
    store_f32(dst + 2 * i, static_cast<float>(u * cs - v * sn));
    store_f32(dst + 2 * i + 1, static_cast<float>(v * cs + u * sn));
    store_f32(dst_v + 2 * i * v_step, 0.f);
    store_f32(dst_v + (2 * i + 1) * v_step, 0.f);
  }
  for (int c = a.n + a.r + tid; c < a.d; c += 256) {
    store_f32(dst + c, 0.f);
    store_f32(dst_v + c * v_step, 0.f);
  }
}

template <typename T, typename Acc>
__global__ void __launch_bounds__(256) turn_pairs_kernel(T* __restrict__ x, int64_t stride, const int32_t* __restrict__ positions, const float* __restrict__ cos_t,
                                                         const float* __restrict__ sin_t, int64_t units, int heads, int head_size, int first, int pairs) {
  const int64_t idx = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (idx >= units) return;
  const int i = static_cast<int>(idx % pairs), h = static_cast<int>(idx / pairs % heads);
  const int64_t t = idx / pairs / heads;
  T* at = x + t * stride + static_cast<int64_t>(h) * head_size + first + 2 * i;
  const int64_t angle = static_cast<int64_t>(positions[t]) * pairs + i;
  const Acc u = static_cast<Acc>(load_f32(at)), v = static_cast<Acc>(load_f32(at + 1)), cs = static_cast<Acc>(cos_t[angle]), sn = static_cast<Acc>(sin_t[angle]);
  store_f32(at, static_cast<float>(u * cs - v * sn));
  store_f32(at + 1, static_cast<float>(v * cs + u * sn));
}

}  // namespace alofa

using namespace alofa;

extern "C" int alofa_latent_rows(const void* x, int64_t x_stride, int dtype, int tokens, int q_at, int q_rank, const float* q_weight, float q_eps, void* cq, int64_t cq_stride,
                                 int kv_at, int r, int n, const float* kv_weight, float kv_eps, const int32_t* positions, const float* cos_t, const float* sin_t,
                                 const int64_t* slots, void* k_cache, void* v_cache, int block_size, int d, void* rows_out, int64_t row_stride, int row_width, int exact,
                                 hipStream_t stream) {
  ALOFA_REQUIRE(tokens >= 0 && r > 0 && n >= 0 && n % 2 == 0 && kv_at >= 0 && kv_at + r + n <= x_stride && kv_weight && kv_eps > 0.f, "latent_rows: bad sizes (r=%d n=%d at=%d stride=%lld)", r, n, kv_at, static_cast<long long>(x_stride));
  ALOFA_REQUIRE(q_rank == 0 || (q_rank > 0 && q_at >= 0 && q_at + q_rank <= x_stride && cq && q_weight && q_eps > 0.f && cq_stride >= q_rank), "latent_rows: the queries' latent does not fit (rank=%d at=%d)", q_rank, q_at);
  ALOFA_REQUIRE(rows_out ? (row_width >= r + n && row_stride >= row_width) : (slots && k_cache && v_cache && block_size > 0 && d >= r + n && (n == 0 || (positions && cos_t && sin_t))),
                "latent_rows: rows of %d values, or pages of keys of %d channels, for %d + %d", row_width, d, r, n);
  ALOFA_REQUIRE(!exact || dtype == kF32, "latent_rows: the exact path is float32");
  if (tokens == 0) return 0;
  LatentRows a{x_stride, q_at, q_rank, q_weight, q_eps, cq_stride, kv_at, r, n, kv_weight, kv_eps, positions, cos_t, sin_t, slots, block_size, d, row_stride, row_width};
  const unsigned grid = static_cast<unsigned>(static_cast<int64_t>(tokens) * (q_rank > 0 ? 2 : 1));
#define ALOFA_LATENT_ROWS(T, ACC) latent_rows_kernel<T, ACC><<<grid, 256, 0, stream>>>(static_cast<const T*>(x), static_cast<T*>(cq), static_cast<T*>(k_cache), static_cast<T*>(v_cache), static_cast<T*>(rows_out), tokens, a)
  if (exact) ALOFA_LATENT_ROWS(float, double);
  else if (dtype == kF32) ALOFA_LATENT_ROWS(float, float);
  else ALOFA_LATENT_ROWS(bf16_t, float);
#undef ALOFA_LATENT_ROWS
  return check_launch("latent_rows");
}

extern "C" int alofa_turn_pairs(void* x, int64_t stride, int dtype, const int32_t* positions, const float* cos_t, const float* sin_t, int tokens, int heads, int head_size,
                                int first, int pairs, int exact, hipStream_t stream) {
  ALOFA_REQUIRE(tokens >= 0 && heads > 0 && pairs > 0 && first >= 0 && first + 2 * pairs <= head_size && static_cast<int64_t>(heads) * head_size <= stride && positions && cos_t && sin_t,
                "turn_pairs: %d pairs from channel %d do not fit a head of %d channels", pairs, first, head_size);
  ALOFA_REQUIRE(!exact || dtype == kF32, "turn_pairs: the exact path is float32");
  if (tokens == 0) return 0;
  const int64_t units = static_cast<int64_t>(tokens) * heads * pairs;
  const unsigned grid = static_cast<unsigned>((units + 255) / 256);
  if (exact) turn_pairs_kernel<float, double><<<grid, 256, 0, stream>>>(static_cast<float*>(x), stride, positions, cos_t, sin_t, units, heads, head_size, first, pairs);
  else if (dtype == kF32) turn_pairs_kernel<float, float><<<grid, 256, 0, stream>>>(static_cast<float*>(x), stride, positions, cos_t, sin_t, units, heads, head_size, first, pairs);
  else turn_pairs_kernel<bf16_t, float><<<grid, 256, 0, stream>>>(static_cast<bf16_t*>(x), stride, positions, cos_t, sin_t, units, heads, head_size, first, pairs);
  return check_launch("turn_pairs");
}
