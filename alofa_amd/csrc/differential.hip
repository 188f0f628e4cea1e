// Attention with two maps per head over the same values, one taken from the other: a head's queries and keys are two halves, each with a softmax
// of its own, and what the head gives is a1 - lambda a2 over its root mean square, times a factor.
//
//   combine_maps          the always-valid end: both maps' sums as float rows, the difference, its norm, the factor.
//   maps_prefill          portions of prompts in bfloat16 on the matrix cores: a wavefront owns 16 rows of one head, with both maps (a tile of values
//                         that is read from LDS then meets four operands: two maps, each weight as two bfloat16 numbers) or with one, and the head's
//                         end is made in registers: one launch from queries to the output product's rows.
// (Single tokens go through the decode kernel of attention_decode.hip, in its form for two maps.)
//
// maps_prefill: a block serves, with TEAMS teams of four or eight wavefronts, 64 consecutive rows of one request and one head. The visible keys are
// walked in tiles of 64 (heads of 256 channels: 32) that start at absolute multiples of their size: first those that hold the sequence's kept first tokens, then the window's;
// the teams take the tiles in turn and their states meet in LDS at the end, in team order. Per tile a team stages
// the keys [tile, d] (a key's two halves side by side) and the values transposed [d, tile].
// Both products are taken transposed (v_mfma_f32_16x16x32_bf16; lane l: A row and B column l % 16, reduction slots 8 (l / 16) .. + 7, D column
// l % 16 and rows 4 (l / 16) .. + 3), so a lane stays with one query row:
//   S_m^T[key, q] = K_m[key, :] . Q_m[q, :]     A = keys from LDS, B = queries (registers)
//   O_m^T[c, q] += V^T[c, key] * P_m^T[key, q]   A = values from LDS, B = weights (registers)
// Scores, weights and their sums are float. A cap of scores, cap tanh(s / cap), takes one exponential and one reciprocal more per score. Scores
// that a cap keeps within +-80 (in units of log2 e) need no running maximum: their weights are exp2(score) as they are, and nothing is rescaled on the way.
// Cache: keys [page, 2 kv_heads, slot, d / 2] (head by head map 1, map 2), values transposed [page, kv_heads, d, slot].
#include "common.h"

#include <float.h>

namespace alofa {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr float kLog2e = 1.44269504088896340736f;

// A wavefront per (row, head); rows: the rows that are served (null: all).
template <typename T, typename Acc>
__global__ void __launch_bounds__(256) combine_maps_kernel(T* __restrict__ out, int64_t out_stride, const float* __restrict__ a, int64_t a_stride, const int32_t* __restrict__ rows, int64_t units,
                                                           int heads, int d, int d_true, float lambda, float gain, float eps) {
  const int64_t unit = static_cast<int64_t>(blockIdx.x) * 4 + threadIdx.x / kWave;
  if (unit >= units) return;
  const int lane = threadIdx.x % kWave;
  const int64_t t = rows ? rows[unit / heads] : unit / heads;
  const int h = static_cast<int>(unit % heads);
  const float* a1 = a + t * a_stride + static_cast<int64_t>(2 * h) * d;
  const float* a2 = a1 + d;
  constexpr int kOwn = 4;      // heads up to 256 channels
  Acc o[kOwn], ss = 0;
#pragma unroll
  for (int n = 0; n < kOwn; ++n) {
    const int c = lane + n * kWave;
    o[n] = c < d_true ? static_cast<Acc>(a1[c]) - static_cast<Acc>(lambda) * static_cast<Acc>(a2[c]) : Acc(0);
    ss += o[n] * o[n];
  }
  ss = wave_sum(ss);
  const Acc f = static_cast<Acc>(gain) / sqrt(ss / static_cast<Acc>(d_true) + static_cast<Acc>(eps));
  T* dst = out + t * out_stride + static_cast<int64_t>(h) * d;
#pragma unroll
  for (int n = 0; n < kOwn; ++n) {
    const int c = lane + n * kWave;
    if (c < d) store_f32(dst + c, static_cast<float>(o[n] * f));
  }
}

constexpr int kPad = 8;

struct MapsArgs {
  int64_t out_stride, q_stride;
  const int32_t* table;
  int max_blocks;
  const int32_t* tiles;      // [blocks, 4]: request, first row, rows (<= 64), position of the first row
  int heads, kv_heads, bs_shift, window, keep_first, d_true;
  float scale, cap, lambda, gain, eps;
};

// NM: maps a wavefront owns. 2: both, four wavefronts a team. 1: one, eight wavefronts a team; the second map's sums go through LDS at the end.
// kCap: 0 scores as they are; 1 capped, with a running maximum; 2 capped so that no maximum is needed
template <int DT, int TEAMS, int kTileKeys, int NM, int kCap>
__global__ void __launch_bounds__(512 / NM * TEAMS, (NM == 1 && DT <= 8) ? 4 : 1) maps_prefill_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ q, const bf16_t* __restrict__ k_cache,
                                                                   const bf16_t* __restrict__ v_cache, MapsArgs a) {
  constexpr int d = DT * 16, dm = d / 2, DS = (dm + 31) / 32;
  constexpr int KQ = kTileKeys / 16, KH = kTileKeys / 32;      // quarters of 16 keys for the first product, halves of 32 for the second
  constexpr int KROW = d + kPad, VROW = kTileKeys + kPad;
  constexpr int kStageBytes = ((kTileKeys * KROW + d * VROW) * 2 + 15) / 16 * 16;
  constexpr int kStateFloats = 2 * 4 * DT + 4;      // per lane: two maxima, two sums, two maps' channels
  constexpr int kTeam = 512 / NM;                   // threads of a team
  static_assert(NM == 2 || TEAMS == 1, "one map a wavefront: one team");
  constexpr int kStateBytes = NM == 2 ? (TEAMS - 1) * 256 * kStateFloats * 4 : 256 * (4 * DT + 1) * 4;
  constexpr int kRoom = TEAMS * kStageBytes > kStateBytes ? TEAMS * kStageBytes : kStateBytes;
  __shared__ __attribute__((aligned(16))) char room[kRoom];
  const int wave_of_block = __builtin_amdgcn_readfirstlane(threadIdx.x / 64);
  const int team = wave_of_block / (8 / NM), wave = wave_of_block % 4, lane = threadIdx.x % 64, tid = threadIdx.x % kTeam;
  const int own = NM == 2 ? 0 : wave_of_block / 4;      // the (first) map of this wavefront
  bf16_t* Ks = reinterpret_cast<bf16_t*>(room + team * kStageBytes);
  bf16_t* Vt = Ks + kTileKeys * KROW;
  const int c16 = lane % 16, g = lane / 16;
  const int head = blockIdx.y, hk = head / (a.heads / a.kv_heads);
  const int32_t* tile = a.tiles + 4 * static_cast<int64_t>(blockIdx.x);
  const int row0 = tile[1], n_rows = tile[2], pos0 = tile[3];
  const int32_t* table = a.table + static_cast<int64_t>(tile[0]) * a.max_blocks;
  const int W = a.window, my_row = wave * 16 + c16, my_pos = pos0 + my_row;
  const bool row_ok = my_row < n_rows;

  bf16x8 qf[NM][DS];
#pragma unroll
  for (int m = 0; m < NM; ++m)
#pragma unroll
    for (int ds = 0; ds < DS; ++ds) {
      uint4 v = make_uint4(0, 0, 0, 0);
      const int c = ds * 32 + g * 8;
      if (row_ok && c < dm) v = *reinterpret_cast<const uint4*>(q + static_cast<int64_t>(row0 + my_row) * a.q_stride + static_cast<int64_t>(2 * head + own + m) * dm + c);
      qf[m][ds] = __builtin_bit_cast(bf16x8, v);
    }
  f32x4 o[NM][DT];
#pragma unroll
  for (int m = 0; m < NM; ++m)
#pragma unroll
    for (int nt = 0; nt < DT; ++nt) o[m][nt] = f32x4{0.f, 0.f, 0.f, 0.f};
  float top[NM], l[NM];
#pragma unroll
  for (int m = 0; m < NM; ++m) top[m] = -FLT_MAX, l[m] = 0.f;
  const float scale2 = a.scale * kLog2e;                       // scores in units of log2 e
  const float inner = kCap ? 2.f * scale2 / a.cap : 0.f;       // exp(2 s / cap) = exp2(inner * product)
  const float cap2 = a.cap * kLog2e;

  // the keys the block needs: [0, keep) and [first_key, last_pos]; index i of its tiles: first those of the kept tokens, then the window's
  const int last_pos = pos0 + n_rows - 1;
  const int first_key = (W > 0 && pos0 - W + 1 > 0) ? pos0 - W + 1 : 0;
  const int keep = W > 0 ? min(a.keep_first, last_pos + 1) : 0;
  const int keep_tiles = (keep + kTileKeys - 1) / kTileKeys;
  const int w_begin = max(first_key / kTileKeys, keep_tiles), w_end = last_pos / kTileKeys;
  const int n_tiles = keep_tiles + max(0, w_end - w_begin + 1);
  auto tile_of = [&](int i) { return i < keep_tiles ? i : w_begin + i - keep_tiles; };

  // Staging as in attention_prefill.hip: 16-byte chunks (eight channels of a key, eight keys of a channel); every lane issues every load, from a key
  // whose page is held in place of one that is not seen, and what such a load brings is cleared.
  constexpr int kChunks = kTileKeys * d / 8;
  constexpr int kPerThread = (kChunks + kTeam - 1) / kTeam;
  const int page_mask = (1 << a.bs_shift) - 1;
  const int v_first = first_key & ~7, v_last = last_pos & ~7;
  uint4 k_reg[kPerThread], v_reg[kPerThread];
  int k_page[kPerThread], v_page[kPerThread];
  auto chunk_of = [&](int j) { const int c = tid + kTeam * j; return c < kChunks ? c : kChunks - 1; };
  auto held = [&](int key, int lo, int hi) { return key < keep ? key : (key < lo ? lo : (key > hi ? hi : key)); };
  auto k_key = [&](int t, int j) { return t * kTileKeys + chunk_of(j) / (d / 8); };
  auto v_key0 = [&](int t, int j) { return t * kTileKeys + (chunk_of(j) % (kTileKeys / 8)) * 8; };
  auto lookup = [&](int t) {
#pragma unroll
    for (int j = 0; j < kPerThread; ++j) {
      k_page[j] = table[held(k_key(t, j), first_key, last_pos) >> a.bs_shift];
      v_page[j] = table[held(v_key0(t, j), v_first, v_last) >> a.bs_shift];
    }
  };
  auto fetch = [&](int t) {
#pragma unroll
    for (int j = 0; j < kPerThread; ++j) {
      const int c = chunk_of(j), ch = (c % (d / 8)) * 8, m = ch >= dm ? 1 : 0;
      const int key = held(k_key(t, j), first_key, last_pos);
      k_reg[j] = *reinterpret_cast<const uint4*>(k_cache + ((((static_cast<int64_t>(k_page[j]) * 2 * a.kv_heads + 2 * hk + m) << a.bs_shift) + (key & page_mask)) * dm) + ch - m * dm);
    }
#pragma unroll
    for (int j = 0; j < kPerThread; ++j) {
      const int key0 = held(v_key0(t, j), v_first, v_last), channel = chunk_of(j) / (kTileKeys / 8);
      v_reg[j] = *reinterpret_cast<const uint4*>(v_cache + (((static_cast<int64_t>(v_page[j]) * a.kv_heads + hk) * d + channel) << a.bs_shift) + (key0 & page_mask));
    }
  };
  auto stage = [&](int t) {
    const int t0 = t * kTileKeys;
    const bool whole = (t0 >= first_key || t0 + kTileKeys <= keep) && t0 + kTileKeys - 1 <= last_pos;      // uniform over the team
#pragma unroll
    for (int j = 0; j < kPerThread; ++j) {
      const int c = tid + kTeam * j;
      if (c >= kChunks) continue;
      uint4 kv = k_reg[j], vv = v_reg[j];
      if (!whole) {
        auto seen = [&](int key) { return (key < keep || key >= first_key) && key <= last_pos; };
        const uint32_t kk = 0u - static_cast<uint32_t>(seen(k_key(t, j)));
        kv = make_uint4(kv.x & kk, kv.y & kk, kv.z & kk, kv.w & kk);
        const int key0 = v_key0(t, j);
        uint32_t w[4] = {vv.x, vv.y, vv.z, vv.w};
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const uint32_t on = 0u - static_cast<uint32_t>(seen(key0 + e));
          w[e / 2] &= (e % 2) ? (on << 16) | 0x0000ffffu : on | 0xffff0000u;
        }
        vv = make_uint4(w[0], w[1], w[2], w[3]);
      }
      *reinterpret_cast<uint4*>(&Ks[(c / (d / 8)) * KROW + (c % (d / 8)) * 8]) = kv;
      // (groups of four keys of a row are permuted by the row's number / 8, so that rows r and r + 8 meet different banks)
      const int row = c / (kTileKeys / 8), sw = (row >> 3) & 7;
      if (sw & 1) vv = make_uint4(vv.z, vv.w, vv.x, vv.y);
      *reinterpret_cast<uint4*>(&Vt[row * VROW + ((((c % (kTileKeys / 8)) * 2) ^ (sw & 6)) << 2)]) = vv;
    }
  };

  lookup(tile_of(min(team, n_tiles - 1)));
  fetch(tile_of(min(team, n_tiles - 1)));
  lookup(tile_of(min(team + TEAMS, n_tiles - 1)));
  for (int i0 = 0; i0 < n_tiles; i0 += TEAMS) {     // uniform over the block
    const int i = i0 + team;
    const bool mine = i < n_tiles;
    const int t = tile_of(mine ? i : 0), t0 = t * kTileKeys;
    __syncthreads();      // the previous tile has been read by every wave
    if (mine) stage(t);
    __syncthreads();
    if (!mine) continue;
    fetch(tile_of(min(i + TEAMS, n_tiles - 1)));
    lookup(tile_of(min(i + 2 * TEAMS, n_tiles - 1)));

    // every row of the block sees every key of the tile: no masks
    const bool whole = t0 + kTileKeys - 1 <= pos0 && (W <= 0 || t0 > last_pos - W || t0 + kTileKeys <= keep);
    bf16x8 pf[NM][KH], pl[NM][KH];
    float corr[NM];
#pragma unroll
    for (int m = 0; m < NM; ++m) {
      f32x4 s[KQ];
#pragma unroll
      for (int kt = 0; kt < KQ; ++kt) {
        s[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ds = 0; ds < DS; ++ds) {
          const int c = ds * 32 + g * 8;
          uint4 kv = make_uint4(0, 0, 0, 0);
          if (c < dm) kv = *reinterpret_cast<const uint4*>(&Ks[(kt * 16 + c16) * KROW + (own + m) * dm + c]);
          s[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, kv), qf[m][ds], s[kt], 0, 0, 0);
        }
        if constexpr (DT > 8 || NM == 1) __builtin_amdgcn_sched_barrier(0);
      }
      float p[4 * KQ];
#pragma unroll
      for (int e = 0; e < 4 * KQ; ++e) {
        const float x = s[e / 4][e % 4];
        // cap tanh(s / cap) = cap - 2 cap / (exp(2 s / cap) + 1)
        p[e] = kCap ? __builtin_fmaf(-2.f * cap2, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(inner * x) + 1.f), cap2) : x * scale2;
      }
      if (!whole) {
#pragma unroll
        for (int e = 0; e < 4 * KQ; ++e) {
          const int key = t0 + (e / 4) * 16 + g * 4 + e % 4;
          if (!(key <= my_pos && (W <= 0 || key > my_pos - W || key < keep))) p[e] = -FLT_MAX;
        }
      }
      float sum = 0.f;
      if constexpr (kCap == 2) {
        corr[m] = 1.f;
#pragma unroll
        for (int e = 0; e < 4 * KQ; ++e) {
          p[e] = __builtin_amdgcn_exp2f(p[e]);      // (a masked score is -FLT_MAX: its weight is zero)
          sum += p[e];
        }
        l[m] += sum;
      } else {
        float most = -FLT_MAX;
#pragma unroll
        for (int e = 0; e < 4 * KQ; ++e) most = fmaxf(most, p[e]);
        most = rows_max(most);     // over the four lanes that share the row
        const float m_new = fmaxf(top[m], most);
        corr[m] = __builtin_amdgcn_exp2f(top[m] - m_new);    // 1 while nothing was seen yet (both -FLT_MAX)
        top[m] = m_new;
#pragma unroll
        for (int e = 0; e < 4 * KQ; ++e) {
          p[e] = p[e] > -FLT_MAX ? __builtin_amdgcn_exp2f(p[e] - m_new) : 0.f;
          sum += p[e];
        }
        l[m] = l[m] * corr[m] + sum;   // this lane's share of the row's sum; the four lanes of a row meet at the end
      }
#pragma unroll
      for (int half = 0; half < KH; ++half) {
        const float* ph = p + 8 * half;
        const uint4 w = make_uint4(pack_bf16x2(ph[0], ph[1]), pack_bf16x2(ph[2], ph[3]), pack_bf16x2(ph[4], ph[5]), pack_bf16x2(ph[6], ph[7]));
        pf[m][half] = __builtin_bit_cast(bf16x8, w);
        const uint4 r = make_uint4(pack_bf16x2_rest(ph[0], ph[1], w.x), pack_bf16x2_rest(ph[2], ph[3], w.y), pack_bf16x2_rest(ph[4], ph[5], w.z), pack_bf16x2_rest(ph[6], ph[7], w.w));
        pl[m][half] = __builtin_bit_cast(bf16x8, r);
      }
    }
#pragma unroll
    for (int nt = 0; nt < DT; ++nt) {
      if constexpr (kCap != 2) {
#pragma unroll
        for (int m = 0; m < NM; ++m) o[m][nt] *= corr[m];
      }
      // (row nt * 16 + c16 and its permutation of the four-key groups, which comes round every four tiles of channels: wide heads keep four addresses, not all)
      constexpr int kRound = (DT > 8 || (NM == 1 && DT >= 4)) ? 4 : DT;
      const bf16_t* vrow = Vt + (nt % kRound * 16 + c16) * VROW;
      const int sw = ((nt % kRound * 2 + (c16 >> 3)) & 7) << 2, on = nt / kRound * kRound * 16 * VROW;
#pragma unroll
      for (int half = 0; half < KH; ++half) {
        const uint2 lo = *reinterpret_cast<const uint2*>(vrow + ((half * 32 + g * 4) ^ sw) + on);
        const uint2 hi = *reinterpret_cast<const uint2*>(vrow + ((half * 32 + 16 + g * 4) ^ sw) + on);
        const bf16x8 vv = __builtin_bit_cast(bf16x8, make_uint4(lo.x, lo.y, hi.x, hi.y));
#pragma unroll
        for (int m = 0; m < NM; ++m) o[m][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, pf[m][half], o[m][nt], 0, 0, 0);
#pragma unroll
        for (int m = 0; m < NM; ++m) o[m][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, pl[m][half], o[m][nt], 0, 0, 0);
      }
      if constexpr (DT > 8 || NM == 1) __builtin_amdgcn_sched_barrier(0);      // (operands read far ahead of their use would not fit the registers)
    }
  }

#pragma unroll
  for (int m = 0; m < NM; ++m) l[m] = rows_sum(l[m]);
  if constexpr (TEAMS > 1) {
    // the other teams leave their states where the tiles were; team 0 adds them in team order
    __syncthreads();      // every tile has been read
    float* states = reinterpret_cast<float*>(room);      // [team - 1][value][thread]
    constexpr int kOne = 256 * kStateFloats;
    if (team > 0) {
      float* mine = states + (team - 1) * kOne + tid;
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        mine[(2 * m) * 256] = top[m];
        mine[(2 * m + 1) * 256] = l[m];
#pragma unroll
        for (int nt = 0; nt < DT; ++nt)
#pragma unroll
          for (int e = 0; e < 4; ++e) mine[(4 + (m * DT + nt) * 4 + e) * 256] = o[m][nt][e];
      }
    }
    __syncthreads();
    if (team > 0) return;
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      float big = top[m];
#pragma unroll
      for (int k = 0; k < TEAMS - 1; ++k) big = fmaxf(big, states[k * kOne + tid + (2 * m) * 256]);
      const float e0 = kCap == 2 ? 1.f : __builtin_amdgcn_exp2f(top[m] - big);
      l[m] *= e0;
#pragma unroll
      for (int nt = 0; nt < DT; ++nt) o[m][nt] *= e0;
#pragma unroll
      for (int k = 0; k < TEAMS - 1; ++k) {
        const float* other = states + k * kOne + tid;
        const float e = kCap == 2 ? 1.f : __builtin_amdgcn_exp2f(other[(2 * m) * 256] - big);
        l[m] += other[(2 * m + 1) * 256] * e;
#pragma unroll
        for (int nt = 0; nt < DT; ++nt)
#pragma unroll
          for (int x = 0; x < 4; ++x) o[m][nt][x] += other[(4 + (m * DT + nt) * 4 + x) * 256] * e;
      }
    }
  }
  float l2 = l[NM - 1];
  float* second = reinterpret_cast<float*>(room) + wave * 64 + lane;      // NM 1: [value][row group][lane], what the second map's wavefronts hand over
  if constexpr (NM == 1) {
    __syncthreads();      // every tile has been read
    if (own == 1) {
      second[0] = l[0];
#pragma unroll
      for (int nt = 0; nt < DT; ++nt)
#pragma unroll
        for (int e = 0; e < 4; ++e) second[(1 + nt * 4 + e) * 256] = o[0][nt][e];
    }
    __syncthreads();
    if (own == 1) return;
    l2 = second[0];
  }
  // the head's end: the difference, its root mean square over the row's channels (four lanes hold a row), the factor
  const float i1 = 1.f / l[0], i2 = a.lambda / l2;
  float ss = 0.f;
#pragma unroll
  for (int nt = 0; nt < DT; ++nt)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float y = o[0][nt][e] * i1 - (NM == 2 ? o[NM - 1][nt][e] : second[(1 + nt * 4 + e) * 256]) * i2;
      o[0][nt][e] = y;
      ss += y * y;
    }
  ss = rows_sum(ss);
  if (!row_ok) return;
  const float f = a.gain / sqrtf(ss / static_cast<float>(a.d_true) + a.eps);
  bf16_t* dst = out + static_cast<int64_t>(row0 + my_row) * a.out_stride + static_cast<int64_t>(head) * d + 4 * g;
#pragma unroll
  for (int nt = 0; nt < DT; ++nt)
    *reinterpret_cast<uint2*>(dst + nt * 16) = make_uint2(pack_bf16x2(o[0][nt][0] * f, o[0][nt][1] * f), pack_bf16x2(o[0][nt][2] * f, o[0][nt][3] * f));
}

template <int DT, int TEAMS, int KT = 64, int NM = 2>
static void launch_maps(dim3 grid, hipStream_t stream, void* out, const void* q, const void* k_cache, const void* v_cache, const MapsArgs& a) {
#define ALOFA_MAPS(CAP) maps_prefill_kernel<DT, TEAMS, KT, NM, CAP><<<grid, 512 / NM * TEAMS, 0, stream>>>(static_cast<bf16_t*>(out), static_cast<const bf16_t*>(q), static_cast<const bf16_t*>(k_cache), static_cast<const bf16_t*>(v_cache), a)
  if (a.cap <= 0.f) ALOFA_MAPS(0);
  else if (a.cap * kLog2e > 80.f) ALOFA_MAPS(1);
  else ALOFA_MAPS(2);
#undef ALOFA_MAPS
}

}  // namespace alofa

using namespace alofa;

extern "C" int alofa_combine_maps(void* out, int64_t out_stride, int dtype, const float* a, int64_t a_stride, const int32_t* rows, int tokens, int heads, int d, int d_true, float lambda,
                                  float gain, float eps, int exact, hipStream_t stream) {
  ALOFA_REQUIRE(tokens >= 0 && heads > 0 && d > 0 && d <= 256 && d_true > 0 && d_true <= d, "combine_maps: tokens=%d heads=%d d=%d (up to 256) of which %d count", tokens, heads, d, d_true);
  ALOFA_REQUIRE(out_stride >= static_cast<int64_t>(heads) * d && a_stride >= static_cast<int64_t>(2 * heads) * d, "combine_maps: rows are shorter than their heads");
  ALOFA_REQUIRE(!exact || dtype == kF32, "combine_maps: the exact path is float32");
  if (tokens == 0) return 0;
  const int64_t units = static_cast<int64_t>(tokens) * heads;
  const unsigned grid = static_cast<unsigned>((units + 3) / 4);
#define ALOFA_COMBINE(T, ACC) combine_maps_kernel<T, ACC><<<grid, 256, 0, stream>>>(static_cast<T*>(out), out_stride, a, a_stride, rows, units, heads, d, d_true, lambda, gain, eps)
  if (exact) ALOFA_COMBINE(float, double);
  else if (dtype == kF32) ALOFA_COMBINE(float, float);
  else ALOFA_COMBINE(bf16_t, float);
#undef ALOFA_COMBINE
  return check_launch("combine_maps");
}

extern "C" int alofa_maps_prefill_supports(int d) { return d == 16 || d == 32 || d == 48 || d == 64 || d == 96 || d == 128 || d == 192 || d == 256; }

// bfloat16. d: a value head's channels as stored, and both halves of a query or key head together. lambda, gain, eps: the head's end.
extern "C" int alofa_maps_prefill(void* out, int64_t out_stride, const void* q, int64_t q_stride, const void* k_cache, const void* v_cache, const int32_t* table, int max_blocks,
                                  const int32_t* tiles, int n_tiles, int heads, int kv_heads, int d, int d_true, int block_size, int window, int keep_first, float scale,
                                  float cap, float lambda, float gain, float eps, hipStream_t stream) {
  ALOFA_REQUIRE(n_tiles > 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0, "maps_prefill: tiles=%d heads=%d kv_heads=%d (kv_heads must divide heads)", n_tiles, heads, kv_heads);
  ALOFA_REQUIRE(alofa_maps_prefill_supports(d) && d_true > 0 && d_true <= d, "maps_prefill: head size %d (of which %d count) is not built", d, d_true);
  ALOFA_REQUIRE(block_size >= 8 && (block_size & (block_size - 1)) == 0 && max_blocks > 0 && window >= 0 && keep_first >= 0 && cap >= 0.f,
                "maps_prefill: pages of a power of two of at least 8 tokens (block_size=%d), window=%d keep_first=%d cap=%g", block_size, window, keep_first, cap);
  ALOFA_REQUIRE(q_stride % 8 == 0 && out_stride % 4 == 0 && reinterpret_cast<uintptr_t>(q) % 16 == 0 && reinterpret_cast<uintptr_t>(out) % 8 == 0, "maps_prefill: rows must be 16-byte aligned");
  int shift = 0;
  while ((1 << shift) < block_size) ++shift;
  const MapsArgs a{out_stride, q_stride, table, max_blocks, tiles, heads, kv_heads, shift, window, keep_first, d_true, scale, cap, lambda, gain, eps};
  const dim3 grid(n_tiles, heads);
  // Which form (2,048 rows of 2,048 channels, a window of 1,024, scores capped at 50, us a layer, and the other form's): one map a wavefront where that leaves room for four
  // wavefronts a SIMD (size 32: 181 against 200, 48: 149 against 191, 64: 107 against 125) or where two maps do not fit the registers (192: 116 against 184, 256:
  // 83 against 185); both maps at 96 and 128 channels (117 and 88 against 134 and 96), whose values are then read from LDS once for both.
  switch (d / 16) {
    case 1: launch_maps<1, 1, 64, 1>(grid, stream, out, q, k_cache, v_cache, a); break;
    case 2: launch_maps<2, 1, 64, 1>(grid, stream, out, q, k_cache, v_cache, a); break;
    case 3: launch_maps<3, 1, 64, 1>(grid, stream, out, q, k_cache, v_cache, a); break;
    case 4: launch_maps<4, 1, 64, 1>(grid, stream, out, q, k_cache, v_cache, a); break;
    case 6: launch_maps<6, 2>(grid, stream, out, q, k_cache, v_cache, a); break;
    case 8: launch_maps<8, 2>(grid, stream, out, q, k_cache, v_cache, a); break;
    case 12: launch_maps<12, 1, 64, 1>(grid, stream, out, q, k_cache, v_cache, a); break;
    case 16: launch_maps<16, 1, 32, 1>(grid, stream, out, q, k_cache, v_cache, a); break;
  }
  return check_launch("maps_prefill");
}
