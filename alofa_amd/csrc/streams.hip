// Several copies of the residual stream side by side: x[t, s, :] for s = 0 .. S - 1 (float32), which every sub-layer reads as one weighted sum
// and writes by mixing.
//
//   streams_step   with y [T, h], what a sub-layer gave: x'[t, v] = sum_s mix[s, v] x[t, s] + w_out[v] y[t], all copies at once from the old
//                  ones; without y: x' = x. Then, where somebody reads next, r[t] = sum_v w_in[v] x'[t, v], through an RMS norm with a
//                  weight (or as it is), to rows of the reader's type. `source` [T, h]: every x[t, s] is source[t] (the first step of a
//                  pass: the copies are spread and read in one launch). The copies are stored only where asked for.
//
// Instead of y there may be the results of a mixture of experts slot by slot (grouped.hip): y[t] is then the sum over row t's slots, its place in the
// shared expert's and, where experts hand the row on, weight * row, formed here in the order of `experts_sum`.
//
// A block per row; a thread takes kVec neighbouring channels of all copies at a time, kOwn such runs in registers with their loads on their
// way together, so a row is read once, written once and normed from registers. Rows longer than the registers hold are walked in a loop and the
// sum for the norm is formed again from the copies just stored (by the thread that stored them). Products and sums in Acc (double in
// the exact path), in ascending order of the copies.
#include "common.h"

namespace alofa {

struct SlotRows {
  const float* y;                // [slots, h] (null: no slots)
  const int32_t* slot_of;        // [T * top (+ T)]: the slot of row t's k-th choice (-1: none), then of row t's place in the shared expert
  int top, shared, tokens;
  const float* pass_weight;      // [T] or null
  const bf16_t* pass_x;          // [T, h]
  int64_t pass_stride;
};

struct StreamArgs {
  float* x;                // [T, S, h]
  const float* source;     // [T, h] or null
  const float* y;          // [T, h] or null
  const float* mix;        // [S, S], from x to (with y)
  const float* w_out;      // [S] (with y)
  const float* w_in;       // [S] (with out)
  const float* norm_w;     // [h] or null: no norm
  int streams, h, write;
  float eps;
  SlotRows slots;
};

template <typename Acc, typename TO, int SM, int kVec, int kOwn, int kThreads = 256>
__global__ void __launch_bounds__(kThreads) streams_step_kernel(TO* __restrict__ out, StreamArgs a) {
  constexpr int kRun = kThreads * kVec;
  __shared__ Acc meet[kThreads / kWave];
  const int S = a.streams, h = a.h;
  const int64_t t = blockIdx.x;
  float* x = a.x + t * S * h;
  const float* source = a.source ? a.source + t * h : nullptr;
  const float* y = a.y ? a.y + t * h : nullptr;
  const bool slots = a.slots.y != nullptr, adds = y != nullptr || slots;
  Acc m[SM][SM], wo[SM], wi[SM];      // (the same for every thread: scalar loads)
#pragma unroll
  for (int s = 0; s < SM; ++s) {
    wo[s] = (adds && s < S) ? static_cast<Acc>(a.w_out[s]) : Acc(0);
    wi[s] = (out && s < S) ? static_cast<Acc>(a.w_in[s]) : Acc(0);
#pragma unroll
    for (int v = 0; v < SM; ++v) m[s][v] = (adds && s < S && v < S) ? static_cast<Acc>(a.mix[s * S + v]) : Acc(0);
  }
  auto load = [&](const float* p, float (&v)[kVec]) {
    if constexpr (kVec == 4) {
      const float4 f = *reinterpret_cast<const float4*>(p);
      v[0] = f.x, v[1] = f.y, v[2] = f.z, v[3] = f.w;
    } else {
      v[0] = *p;
    }
  };
  // one run of channels from c on: the new copies (stored where asked for) and what the next reader sees of them
  auto step = [&](int c, const float (&old)[SM][kVec], const float (&add)[kVec], Acc (&read)[kVec]) {
#pragma unroll
    for (int e = 0; e < kVec; ++e) read[e] = 0;
#pragma unroll
    for (int v = 0; v < SM; ++v) {
      if (v >= S) continue;
      float now[kVec];
#pragma unroll
      for (int e = 0; e < kVec; ++e) {
        if (adds) {
          Acc n = 0;
#pragma unroll
          for (int s = 0; s < SM; ++s) n += m[s][v] * static_cast<Acc>(old[s][e]);
          now[e] = static_cast<float>(n + wo[v] * static_cast<Acc>(add[e]));
        } else {
          now[e] = old[v][e];
        }
        read[e] += wi[v] * static_cast<Acc>(now[e]);
      }
      if (a.write) {
        float* dst = x + static_cast<int64_t>(v) * h + c;
        if constexpr (kVec == 4) *reinterpret_cast<float4*>(dst) = make_float4(now[0], now[1], now[2], now[3]);
        else *dst = now[0];
      }
    }
  };
  auto fetch = [&](int c, float (&old)[SM][kVec], float (&add)[kVec]) {
#pragma unroll
    for (int s = 0; s < SM; ++s) {
      if (s < S) load(source ? source + c : x + static_cast<int64_t>(s) * h + c, old[s]);
      else
#pragma unroll
        for (int e = 0; e < kVec; ++e) old[s][e] = 0.f;
    }
    if (y) {
      load(y + c, add);
      return;
    }
#pragma unroll
    for (int e = 0; e < kVec; ++e) add[e] = 0.f;
    if (!slots) return;
    const SlotRows& r = a.slots;
    auto slot_at = [&](int k) { return k < r.top ? r.slot_of[t * r.top + k] : (r.shared && k == r.top ? r.slot_of[static_cast<int64_t>(r.tokens) * r.top + t] : -1); };
    for (int k0 = 0; k0 < r.top + r.shared; k0 += 5) {      // (five slots' values on their way together)
      float part[5][kVec];
#pragma unroll
      for (int u = 0; u < 5; ++u) {
        const int slot = slot_at(k0 + u);
        if (slot >= 0) load(r.y + static_cast<int64_t>(slot) * h + c, part[u]);
        else
#pragma unroll
          for (int e = 0; e < kVec; ++e) part[u][e] = 0.f;
      }
#pragma unroll
      for (int u = 0; u < 5; ++u)
#pragma unroll
        for (int e = 0; e < kVec; ++e) add[e] += part[u][e];
    }
    if (r.pass_weight) {
      const float w = r.pass_weight[t];
      const bf16_t* px = r.pass_x + t * r.pass_stride + c;
#pragma unroll
      for (int e = 0; e < kVec; ++e) add[e] += w * bf16_to_f32(px[e]);
    }
  };
  auto put = [&](int c, const Acc (&r)[kVec], Acc factor, const float (&nw)[kVec]) {
    TO* dst = out + t * h + c;
    float v[kVec];
#pragma unroll
    for (int e = 0; e < kVec; ++e) v[e] = static_cast<float>(a.norm_w ? r[e] * factor * static_cast<Acc>(nw[e]) : r[e]);
    if constexpr (kVec == 4 && sizeof(TO) == 2) *reinterpret_cast<uint2*>(dst) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
    else if constexpr (kVec == 4) *reinterpret_cast<float4*>(dst) = make_float4(v[0], v[1], v[2], v[3]);
    else store_f32(dst, v[0]);
  };
  const int c0 = threadIdx.x * kVec;
  if constexpr (kOwn > 0) {
    float old[kOwn][SM][kVec], add[kOwn][kVec], nw[kOwn][kVec];
    Acc read[kOwn][kVec], ss = 0;
#pragma unroll
    for (int i = 0; i < kOwn; ++i)
      if (c0 + i * kRun < h) {
        if (a.norm_w) load(a.norm_w + c0 + i * kRun, nw[i]);      // (the norm's weights set out with the rest)
        fetch(c0 + i * kRun, old[i], add[i]);
      }
#pragma unroll
    for (int i = 0; i < kOwn; ++i)
      if (c0 + i * kRun < h) {
        step(c0 + i * kRun, old[i], add[i], read[i]);
#pragma unroll
        for (int e = 0; e < kVec; ++e) ss += read[i][e] * read[i][e];
      }
    if (!out) return;
    Acc factor = 1;
    if (a.norm_w) factor = static_cast<Acc>(1) / sqrt(block_sum<Acc, kThreads>(ss, meet) / static_cast<Acc>(h) + static_cast<Acc>(a.eps));
#pragma unroll
    for (int i = 0; i < kOwn; ++i)
      if (c0 + i * kRun < h) put(c0 + i * kRun, read[i], factor, nw[i]);
  } else {
    Acc ss = 0;
    for (int c = c0; c < h; c += kRun) {
      float old[SM][kVec], add[kVec];
      Acc read[kVec];
      fetch(c, old, add);
      step(c, old, add, read);
      if (out && !a.norm_w) put(c, read, Acc(1), add);
#pragma unroll
      for (int e = 0; e < kVec; ++e) ss += read[e] * read[e];
    }
    if (!out || !a.norm_w) return;
    const Acc factor = static_cast<Acc>(1) / sqrt(block_sum<Acc, kThreads>(ss, meet) / static_cast<Acc>(h) + static_cast<Acc>(a.eps));
    for (int c = c0; c < h; c += kRun) {      // (the copies as they are now: this thread stored these channels, or nothing changed)
      Acc read[kVec];
#pragma unroll
      for (int e = 0; e < kVec; ++e) read[e] = 0;
#pragma unroll
      for (int v = 0; v < SM; ++v)
        if (v < S) {
          float now[kVec];
          load((source && !a.write) ? source + c : x + static_cast<int64_t>(v) * h + c, now);
#pragma unroll
          for (int e = 0; e < kVec; ++e) read[e] += wi[v] * static_cast<Acc>(now[e]);
        }
      float nw[kVec];
      load(a.norm_w + c, nw);
      put(c, read, factor, nw);
    }
  }
}

template <typename Acc, typename TO, int SM>
static void launch_streams(void* out, const StreamArgs& a, int tokens, hipStream_t stream) {
#define ALOFA_STREAMS(VEC, OWN, THREADS) streams_step_kernel<Acc, TO, SM, VEC, OWN, THREADS><<<tokens, THREADS, 0, stream>>>(static_cast<TO*>(out), a)
  // a run of four channels a thread where a block's threads cover the row; many copies, or double, fill the registers with one run of a small block
  constexpr bool kMany = SM > 4 || sizeof(Acc) > 4;
  if (a.h % 4 != 0) {
    if (a.h <= 256) ALOFA_STREAMS(1, 1, 256);
    else ALOFA_STREAMS(1, 0, 256);
  } else if (a.h <= 1024) ALOFA_STREAMS(4, 1, 256);
  else if (!kMany && a.h <= 2048) ALOFA_STREAMS(4, 1, (kMany ? 256 : 512));
  else if (!kMany && a.h <= 4096) ALOFA_STREAMS(4, (kMany ? 1 : 2), (kMany ? 256 : 512));
  else ALOFA_STREAMS(4, 0, 256);
#undef ALOFA_STREAMS
}

template <typename Acc, typename TO>
static void pick_streams(void* out, const StreamArgs& a, int tokens, hipStream_t stream) {
  switch (a.streams) {
    case 1: launch_streams<Acc, TO, 1>(out, a, tokens, stream); break;
    case 2: launch_streams<Acc, TO, 2>(out, a, tokens, stream); break;
    case 3: launch_streams<Acc, TO, 3>(out, a, tokens, stream); break;
    case 4: launch_streams<Acc, TO, 4>(out, a, tokens, stream); break;
    default:
      if (a.streams <= 8) launch_streams<Acc, TO, 8>(out, a, tokens, stream);
      else launch_streams<Acc, TO, 16>(out, a, tokens, stream);
  }
}

}  // namespace alofa

using namespace alofa;

extern "C" int alofa_streams_step(void* out, int o_dtype, float* x, const float* source, const float* y, const float* mix, const float* w_out, const float* w_in,
                                  const float* norm_w, float eps, int tokens, int streams, int h, int write, const float* slots_y, const int32_t* slot_of, int top, int shared,
                                  const float* pass_weight, const void* pass_x, int64_t pass_stride, int exact, hipStream_t stream) {
  ALOFA_REQUIRE(slots_y == nullptr || (y == nullptr && slot_of && top > 0 && mix && w_out && !exact && (pass_weight == nullptr || pass_x)), "streams_step: slots come in y's place, with weights to add them by");
  ALOFA_REQUIRE(tokens >= 0 && h > 0 && streams >= 1 && streams <= 16, "streams_step: tokens=%d h=%d streams=%d (1 to 16)", tokens, h, streams);
  ALOFA_REQUIRE(x != nullptr && (y == nullptr || (mix && w_out)) && (out == nullptr || w_in), "streams_step: operands are missing");
  ALOFA_REQUIRE(write || (y == nullptr && slots_y == nullptr) || norm_w == nullptr || out == nullptr || h <= 1024, "streams_step: a norm of long rows that are not stored");
  ALOFA_REQUIRE(!exact || out == nullptr || o_dtype == kF32, "streams_step: the exact path is float32");
  if (tokens == 0) return 0;
  const StreamArgs a{x, source, y, mix, w_out, w_in, norm_w, streams, h, write, eps,
                     SlotRows{slots_y, slot_of, top, shared, tokens, pass_weight, static_cast<const bf16_t*>(pass_x), pass_stride}};
  if (exact) pick_streams<double, float>(out, a, tokens, stream);
  else if (o_dtype == kF32) pick_streams<float, float>(out, a, tokens, stream);
  else pick_streams<float, bf16_t>(out, a, tokens, stream);
  return check_launch("streams_step");
}
