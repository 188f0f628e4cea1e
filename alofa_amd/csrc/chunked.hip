// The linear recurrence with one constant decay g per head, for steps of many rows: S_t = g S_(t-1) + k_t v_t^T, o_t = S_t^T q_t, taken
// in chunks of up to 64 rows of one request instead of row by row. With t, s counting a chunk's rows from 0 and n its rows:
//   what the chunk adds      U = sum_s g^(n-1-s) k_s v_s^T                                    (chunk_add: every chunk by itself)
//   the state in front of it S' = g^n S + U                                                   (chunk_states: a request's chunks in order)
//   its read-outs            o_t = g^(t+1) S^T q_t + sum_(s <= t) g^(t-s) (q_t . k_s) v_s     (chunk_read: every chunk by itself)
// All products run in float on the matrix cores (v_mfma_f32_16x16x4_f32: lane l holds A row and B column l % 16 at reduction index l / 16,
// and D column l % 16, rows 4 (l / 16) .. + 3), on operands that are bfloat16 numbers times a power of g, so nothing but float rounding
// separates the result from the recurrence row by row. q, k, v come as bfloat16 rows; the powers g^0 .. g^64 from a table; q is
// scaled by q_scale and k by k_scale.
//
// Chunks: int32 [n_chunks, 4]: request, first row, rows (<= 64), 0; a request's chunks lie together, in its rows' order, and
// of_request [requests, 2] holds the first one's number and their count. added [n_chunks, heads, dk, dv] float: U, then, in its place, the
// state in front of the chunk.
#include "common.h"

namespace alofa {

typedef float chunk_f32x4 __attribute__((ext_vector_type(4)));
constexpr int kChunkRows = 64, kPowers = kChunkRows + 1;

// A block of four wavefronts per (chunk, head, 64 x 64 piece of the state); wavefront w the piece's key channels 16 w .. + 15.
__global__ void __launch_bounds__(256) chunk_add_kernel(float* __restrict__ added, const bf16_t* __restrict__ k, int64_t k_stride, const bf16_t* __restrict__ v, int64_t v_stride,
                                                        const int32_t* __restrict__ chunks, const float* __restrict__ powers, int heads, int dk, int dv, float k_scale, int key_tiles) {
  constexpr int kRow = 80;      // floats of a staged row: rows one apart start 16 banks apart
  __shared__ float ks[kChunkRows][kRow], vs[kChunkRows][kRow];
  const int chunk = blockIdx.x, head = blockIdx.y, c0 = (blockIdx.z % key_tiles) * 64, j0 = (blockIdx.z / key_tiles) * 64;
  const int row0 = chunks[4 * chunk + 1], n = chunks[4 * chunk + 2];
  const float* pow_g = powers + head * kPowers;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
#pragma unroll
  for (int e = 0; e < 16; ++e) {      // (a wavefront brings in one row after the other, a lane a channel; rows past the chunk's end and channels past the head's are zeros)
    const int s = e * 4 + wave;
    const bool in = s < n;
    const int64_t r = row0 + (in ? s : 0);
    const float f = in ? pow_g[n - 1 - s] * k_scale : 0.f;
    ks[s][lane] = (in && c0 + lane < dk) ? bf16_to_f32(k[r * k_stride + static_cast<int64_t>(head) * dk + c0 + lane]) * f : 0.f;
    vs[s][lane] = (in && j0 + lane < dv) ? bf16_to_f32(v[r * v_stride + static_cast<int64_t>(head) * dv + j0 + lane]) : 0.f;
  }
  __syncthreads();
  const int c16 = lane % 16, g = lane / 16;
  chunk_f32x4 acc[4];
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) acc[jt] = chunk_f32x4{0.f, 0.f, 0.f, 0.f};
  const int steps = (n + 3) / 4;
#pragma unroll 4
  for (int st = 0; st < steps; ++st) {
    const float a = ks[4 * st + g][16 * wave + c16];
#pragma unroll
    for (int jt = 0; jt < 4; ++jt) acc[jt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, vs[4 * st + g][16 * jt + c16], acc[jt], 0, 0, 0);
  }
  float* dst = added + (static_cast<int64_t>(chunk) * heads + head) * dk * dv;
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    const int j = j0 + 16 * jt + c16;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = c0 + 16 * wave + 4 * g + i;
      if (c < dk && j < dv) dst[static_cast<int64_t>(c) * dv + j] = acc[jt][i];
    }
  }
}

// A thread per value of a request's state: the chunks in order, eight of them on their way together.
__global__ void __launch_bounds__(256) chunk_states_kernel(float* __restrict__ added, float* __restrict__ state, const int32_t* __restrict__ chunks, const int32_t* __restrict__ of_request,
                                                           const int32_t* __restrict__ req_slot, const float* __restrict__ powers, int heads, int per_head) {
  constexpr int kAhead = 8;
  const int r = blockIdx.y;
  const int64_t width = static_cast<int64_t>(heads) * per_head, e = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
  if (e >= width) return;
  const float* pow_g = powers + static_cast<int>(e / per_head) * kPowers;
  float* mine = state + static_cast<int64_t>(req_slot[r]) * width + e;
  const int first = of_request[2 * r], count = of_request[2 * r + 1];
  float S = *mine;
  for (int c0 = 0; c0 < count; c0 += kAhead) {
    float u[kAhead], f[kAhead];
#pragma unroll
    for (int a = 0; a < kAhead; ++a) {
      const int c = first + (c0 + a < count ? c0 + a : count - 1);
      u[a] = added[static_cast<int64_t>(c) * width + e];
      f[a] = pow_g[chunks[4 * c + 2]];
    }
#pragma unroll
    for (int a = 0; a < kAhead; ++a) {
      if (c0 + a < count) {
        added[static_cast<int64_t>(first + c0 + a) * width + e] = S;
        S = f[a] * S + u[a];
      }
    }
  }
  *mine = S;
}

// A block of four wavefronts per (chunk, head, 64 value channels); wavefront w the chunk's rows 16 w .. + 15.
__global__ void __launch_bounds__(256) chunk_read_kernel(float* __restrict__ out, int64_t out_stride, const bf16_t* __restrict__ q, int64_t q_stride, const bf16_t* __restrict__ k,
                                                         int64_t k_stride, const bf16_t* __restrict__ v, int64_t v_stride, const float* __restrict__ before,
                                                         const int32_t* __restrict__ chunks, const float* __restrict__ powers, int heads, int dk, int dv, float q_scale, float k_scale) {
  // floats of a staged row: values are read in rows four apart, the state's in rows eight apart, by the four rows of lanes: 16 banks apart both ways
  constexpr int kVRow = 68, kSRow = 66;
  __shared__ float vs[kChunkRows][kVRow], ss[64][kSRow];
  const int chunk = blockIdx.x, head = blockIdx.y, j0 = blockIdx.z * 64;
  const int row0 = chunks[4 * chunk + 1], n = chunks[4 * chunk + 2];
  const float* pow_g = powers + head * kPowers;
  const float* S = before + (static_cast<int64_t>(chunk) * heads + head) * dk * dv;
  const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, c16 = lane % 16, g = lane / 16;
  const int t = 16 * wave + c16;            // this lane's query row
  const bool active = 16 * wave < n, t_ok = t < n;
  const bf16_t* q_row = q + static_cast<int64_t>(row0 + (t_ok ? t : 0)) * q_stride + static_cast<int64_t>(head) * dk;
  const float q_front = t_ok ? pow_g[t + 1] * q_scale : 0.f;
#pragma unroll
  for (int e = 0; e < 16; ++e) {
    const int s = e * 4 + wave;
    vs[s][lane] = (s < n && j0 + lane < dv) ? bf16_to_f32(v[static_cast<int64_t>(row0 + s) * v_stride + static_cast<int64_t>(head) * dv + j0 + lane]) : 0.f;
  }
  chunk_f32x4 acc[4];
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) acc[jt] = chunk_f32x4{0.f, 0.f, 0.f, 0.f};
  // eight channels of a row, from channel c on (a head's size is a multiple of eight: all of them or none)
  auto eight = [&](const bf16_t* row, int c, bool ok, float (&x)[8]) {
    uint4 w = make_uint4(0, 0, 0, 0);
    if (ok && c < dk) w = *reinterpret_cast<const uint4*>(row + c);
    const uint32_t p[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) x[2 * i] = __uint_as_float(p[i] << 16), x[2 * i + 1] = __uint_as_float(p[i] & 0xffff0000u);
  };
  // ---- the state in front of the chunk, 64 key channels at a time
  for (int c0 = 0; c0 < dk; c0 += 64) {
    __syncthreads();
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int c = e * 4 + wave;
      ss[c][lane] = (c0 + c < dk && j0 + lane < dv) ? S[static_cast<int64_t>(c0 + c) * dv + j0 + lane] : 0.f;
    }
    __syncthreads();
    if (!active) continue;
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      if (c0 + 32 * half >= dk) break;      // (uniform)
      float x[8];
      eight(q_row, c0 + 32 * half + 8 * g, t_ok, x);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float a = x[i] * q_front;
#pragma unroll
        for (int jt = 0; jt < 4; ++jt) acc[jt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, ss[32 * half + 8 * g + i][16 * jt + c16], acc[jt], 0, 0, 0);
      }
    }
  }
  if (!active) return;
  // ---- the chunk's own rows up to the query: sixteen keys at a time. The products are formed transposed (key rows, query columns): what a lane then holds,
  // query t and keys 4 g + i, is its operand of the products with the values.
  for (int st = 0; st <= wave; ++st) {
    const int s_row = 16 * st + c16;
    const bf16_t* k_row = k + static_cast<int64_t>(row0 + (s_row < n ? s_row : 0)) * k_stride + static_cast<int64_t>(head) * dk;
    chunk_f32x4 p{0.f, 0.f, 0.f, 0.f};
    for (int c0 = 0; c0 < dk; c0 += 32) {
      float x[8], y[8];
      eight(k_row, c0 + 8 * g, s_row < n, x);
      eight(q_row, c0 + 8 * g, t_ok, y);
#pragma unroll
      for (int i = 0; i < 8; ++i) p = __builtin_amdgcn_mfma_f32_16x16x4f32(x[i], y[i], p, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int s = 16 * st + 4 * g + i;
      const float a = (s <= t && t_ok) ? p[i] * (pow_g[t - s] * (q_scale * k_scale)) : 0.f;
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) acc[jt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, vs[s][16 * jt + c16], acc[jt], 0, 0, 0);
    }
  }
#pragma unroll
  for (int jt = 0; jt < 4; ++jt) {
    const int j = j0 + 16 * jt + c16;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 16 * wave + 4 * g + i;
      if (row < n && j < dv) out[static_cast<int64_t>(row0 + row) * out_stride + static_cast<int64_t>(head) * dv + j] = acc[jt][i];
    }
  }
}

}  // namespace alofa

using namespace alofa;

extern "C" int alofa_chunk_rows() { return kChunkRows; }

extern "C" int alofa_chunked_recurrence(float* out, int64_t out_stride, const void* q, int64_t q_stride, const void* k, int64_t k_stride, const void* v, int64_t v_stride, float* state,
                                        const int32_t* req_slot, const int32_t* chunks, int n_chunks, const int32_t* of_request, int requests, const float* powers, float* added,
                                        int heads, int dk, int dv, float q_scale, float k_scale, hipStream_t stream) {
  ALOFA_REQUIRE(n_chunks >= 0 && requests >= 0 && n_chunks >= requests && heads > 0 && dk > 0 && dk % 8 == 0 && dv > 0, "chunked_recurrence: bad sizes (chunks=%d requests=%d heads=%d dk=%d dv=%d; dk a multiple of 8)", n_chunks, requests, heads, dk, dv);
  ALOFA_REQUIRE(q_stride % 8 == 0 && k_stride % 8 == 0 && reinterpret_cast<uintptr_t>(q) % 16 == 0 && reinterpret_cast<uintptr_t>(k) % 16 == 0, "chunked_recurrence: rows of q and k must be 16-byte aligned");
  ALOFA_REQUIRE(heads <= 65535 && requests <= 65535, "chunked_recurrence: %d heads, %d requests", heads, requests);
  if (n_chunks == 0) return 0;
  const int key_tiles = (dk + 63) / 64, value_tiles = (dv + 63) / 64;
  const bf16_t *qb = static_cast<const bf16_t*>(q), *kb = static_cast<const bf16_t*>(k), *vb = static_cast<const bf16_t*>(v);
  chunk_add_kernel<<<dim3(n_chunks, heads, key_tiles * value_tiles), 256, 0, stream>>>(added, kb, k_stride, vb, v_stride, chunks, powers, heads, dk, dv, k_scale, key_tiles);
  if (check_launch("chunked_recurrence (add)")) return 1;
  const int64_t width = static_cast<int64_t>(heads) * dk * dv;
  chunk_states_kernel<<<dim3(static_cast<unsigned>((width + 255) / 256), requests), 256, 0, stream>>>(added, state, chunks, of_request, req_slot, powers, heads, dk * dv);
  if (check_launch("chunked_recurrence (states)")) return 1;
  chunk_read_kernel<<<dim3(n_chunks, heads, value_tiles), 256, 0, stream>>>(out, out_stride, qb, q_stride, kb, k_stride, vb, v_stride, added, chunks, powers, heads, dk, dv, q_scale, k_scale);
  return check_launch("chunked_recurrence (read)");
}
