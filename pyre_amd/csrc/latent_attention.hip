// Softmax attention over one compressed row per token that all query heads share: the row [c | r] of a token is `rank`
// elements c, which serve as key and as value, and `dk - rank` further elements r of the key alone (a part that was
// turned by position). A query of head h is [Wuk_h^T q_h | turned part] of dk elements, so that its product with a row
// is the score of the head's own key; what comes out is the weighted sum of the c. Rows lie in pages
// [pages, 1, page, dk].
//
//   s(i, j) = (q_i . row_j) * scale;  i sees j iff j <= i and (window == 0 or i - j < window)
//   out_i   = sum_j softmax_j(s(i, .)) c_j, with exp(sink[head]) in the denominator if there is a sink
//
// One kernel in two forms. A row tile of the matrix cores is 32 queries: for prompt portions the tokens of a tile
// (up to 32 consecutive tokens of a request) for one head, for single tokens 32 heads of the token. G such row tiles
// share a block and the chunk of 32 keys that it keeps in LDS; SL waves share a row tile: each takes every SL-th step
// of the score's inner product (the parts are added through LDS, in order), turns its share of the chunk's scores into
// weights, which go round through LDS as well, and has NVT * 32 columns of the output. The
// problem is transposed, S^T[key, query] and O^T[d, query], so that a lane's sixteen scores are operands of the second
// product as they are. Scores, maxima, weights and sums are float32, the exponentials base two on scores scaled by
// log2(e). bfloat16 rows and queries go through the 16-bit instruction (a product of two is exact in float32), each
// float32 weight as three bfloat16 pieces that sum to it exactly; float32 rows and queries through the float32
// instruction.
//
// Chunks start at multiples of 32 positions, spans (a single token's keys dealt to several blocks) at multiples of
// `span`: the order of a query's sums follows from its own position alone.
#include "pyre_api.h"
#include "pyre_common.h"
#include "pyre_vec4.h"

using namespace pyre;

namespace {

typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int kKeys = 32;
constexpr int kRing = 4;
constexpr float kLog2e = 1.44269504088896340736f;

struct LatentArgs {
  const void* q;            // [n][heads][dk]
  const void* rows;         // [pages][1][page][dk]
  void* out;                // [n][heads][rank]
  float* part;              // single tokens, several spans: sums [listed][heads][spans][rank], else null
  float* part_ml;           // and behind them maximum and weight [listed][heads][spans][2]
  const int* list;          // tiles (first token, count), or single tokens (null: token = block)
  const int* positions;
  const int* seq_of_token;
  const int* table;
  const float* sink;        // [heads] or null
  int table_stride, heads, rank, dk, page_size, window, span, spans, vec, tab_lds, two_buffers;
  float scale2;             // scale * log2(e)
};

// A barrier that waits for LDS traffic alone: the next chunk's rows stay on their way.
__device__ inline void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

__device__ inline float exp2_hw(float x) { return __builtin_amdgcn_exp2f(x); }

// 1 / denominator for sums made against the maximum m (base two), a sink included.
__device__ inline float latent_factor(float m, float l, const float* sink, int head) {
  if (!sink) return l > 0.f ? 1.f / l : 0.f;
  const float sk = sink[head] * kLog2e, M = fmaxf(m, sk);
  const float a = m == -INFINITY ? 0.f : exp2_hw(m - M);
  return a / (l * a + exp2_hw(sk - M));
}

// A chunk's weights of one row tile on their way to the waves that share it: three bfloat16 pieces of 32 x 32 weights, in
// the order of the second product's operands, or the weights themselves.
template <typename T> constexpr int weight_bytes() { return sizeof(T) == 2 ? 3 * 2048 : 4096; }

// Two weights as three bfloat16 pieces each, which sum to them exactly.
__device__ inline void split_pair(float p0, float p1, uint32_t& w1, uint32_t& w2, uint32_t& w3) {
  w1 = pack_bf16x2(p0, p1);
  const float r0 = p0 - __uint_as_float(w1 << 16), r1 = p1 - __uint_as_float(w1 & 0xffff0000u);
  w2 = pack_bf16x2(r0, r1);
  w3 = pack_bf16x2(r0 - __uint_as_float(w2 << 16), r1 - __uint_as_float(w2 & 0xffff0000u));
}

// Four keys of sixteen neighbouring columns, transposed on the way out of LDS: of each group of sixteen lanes, lane j
// gives the address of four columns 4 (j % 4) .. of key j / 4 and receives column j of the four keys.
__device__ inline uint2 read_transposed(const bf16* p) {
  const auto v = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
      (__attribute__((address_space(3))) s16x4*)(const_cast<bf16*>(p)));
  return __builtin_bit_cast(uint2, v);
}

template <typename T, int G, int SL, int NVT, int KQ, bool SINGLE>
__global__ __launch_bounds__(64 * G * SL, sizeof(T) == 2 && !SINGLE ? 2 : 1) void latent_attn_kernel(const LatentArgs a) {
  constexpr int NT = 64 * G * SL, TPR = NT / kKeys;     // threads that bring one key's row
  constexpr int E = 16 / sizeof(T);                      // elements of a 16-byte unit
  constexpr int KI = (2 * KQ * SL + TPR - 1) / TPR;      // units a thread brings of a row
  extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
  const int steps = (a.dk + 2 * E - 1) / (2 * E), ldk = 2 * E * steps + E;
  T* Ks = reinterpret_cast<T*>(lds_raw);                                   // [1 or 2][32][ldk], then slack
  const int buffer = kKeys * ldk, slack = max(0, 32 * NVT * SL - ldk);
  const int k_elems = ((a.two_buffers ? 2 : 1) * buffer + slack + 7) / 8 * 8;
  float* sred = reinterpret_cast<float*>(Ks + k_elems);                    // [G * SL][16][64] if SL > 1
  unsigned char* Ps = reinterpret_cast<unsigned char*>(sred + (SL > 1 ? G * SL * 1024 : 0));  // [G] x weight_bytes<T>() if SL > 1
  int* tab_s = reinterpret_cast<int*>(Ps + (SL > 1 ? G * weight_bytes<T>() : 0));
  __shared__ int slot_s[kRing][kKeys];
  __shared__ float row_s[G * SL][32];  // the waves' maxima of their keys, per query; at the end their weights

  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = lane >> 5, c = lane & 31;
  const int g = wave / SL, sl = wave % SL;
  int t0, ntok = 1;
  if (SINGLE) {
    t0 = a.list ? a.list[blockIdx.x] : blockIdx.x;
  } else {
    t0 = a.list[2 * blockIdx.y], ntok = a.list[2 * blockIdx.y + 1];
    if (ntok <= 0) return;
  }
  const int pos0 = a.positions[t0];
  const int* table = a.table + static_cast<size_t>(a.seq_of_token[t0]) * a.table_stride;
  // this lane's query
  const int head = SINGLE ? (blockIdx.y * G + g) * 32 + c : blockIdx.x * G + g;
  const int token = SINGLE ? t0 : t0 + c;
  const bool active = SINGLE ? (blockIdx.y * G + g) * 32 < a.heads : head < a.heads;  // the whole row tile
  const bool live = active && (SINGLE ? head < a.heads : c < ntok);
  const auto first_seen = [&](int pos) { return a.window > 0 ? max(0, pos - a.window + 1) : 0; };
  const int hi = SINGLE || c >= ntok ? pos0 : pos0 + c, lo = first_seen(hi);
  const int lo_tile = first_seen(pos0), hi_tile = pos0 + ntok - 1;
  int lo_all = lo_tile, hi_all = hi_tile;
  if (SINGLE && a.span > 0) {
    const int s0 = (lo_tile / a.span + static_cast<int>(blockIdx.z)) * a.span;
    lo_all = max(lo_all, s0), hi_all = min(hi_all, s0 + a.span - 1);
    if (lo_all > hi_all) return;
  }
  const int chunk0 = lo_all / kKeys, n_chunks = hi_all / kKeys - chunk0 + 1;
  const int last_tile = (a.rank - 1) / 32;
  const int lo_last = first_seen(hi_tile);  // a chunk from here to pos0 is seen whole by every query

  const int entry0 = lo_all / a.page_size;
  if (a.tab_lds)
    for (int i = tid; i < min(a.tab_lds, hi_all / a.page_size - entry0 + 1); i += NT)
      tab_s[i] = entry0 + i < a.table_stride ? table[entry0 + i] : -1;

  uint4 qf[KQ];
  {
    const T* qrow = static_cast<const T*>(a.q) + (static_cast<size_t>(token) * a.heads + head) * a.dk;
#pragma unroll
    for (int st = 0; st < KQ; ++st) {
      const int e0 = 2 * E * (st * SL + sl) + E * h;
      qf[st] = uint4{0u, 0u, 0u, 0u};
      if (!live || e0 >= a.dk) continue;
      if (a.vec) {
        qf[st] = *reinterpret_cast<const uint4*>(qrow + e0);
      } else {
        uint32_t w[4] = {0u, 0u, 0u, 0u};
#pragma unroll
        for (int u = 0; u < E; ++u)
          if (e0 + u < a.dk) {
            if constexpr (sizeof(T) == 4) w[u] = __builtin_bit_cast(uint32_t, qrow[e0 + u]);
            else w[u >> 1] |= static_cast<uint32_t>(__builtin_bit_cast(uint16_t, qrow[e0 + u])) << (16 * (u & 1));
          }
        qf[st] = uint4{w[0], w[1], w[2], w[3]};
      }
    }
  }
  __syncthreads();  // the table is in LDS

  auto slot_of = [&](int key) {
    if (key < lo_all || key > hi_all) return -1;
    const int entry = key / a.page_size;
    if (entry >= a.table_stride) return -1;
    const int page = a.tab_lds ? tab_s[entry - entry0] : table[entry];
    return page < 0 ? -1 : page * a.page_size + key % a.page_size;
  };
  const int my_row = tid / TPR, my_unit = tid % TPR;
  uint4 reg[KI];
  int reg_slot = -1;
  auto ask = [&](int it) {
    reg_slot = slot_s[it % kRing][my_row];
    if (!a.vec) return;
    const uint4* src = reinterpret_cast<const uint4*>(static_cast<const T*>(a.rows) + static_cast<size_t>(max(reg_slot, 0)) * a.dk);
#pragma unroll
    for (int k = 0; k < KI; ++k) {
      const int unit = my_unit + k * TPR;
      reg[k] = uint4{0u, 0u, 0u, 0u};
      if (reg_slot >= 0 && unit * E < a.dk) reg[k] = src[unit];
    }
  };
  auto stash = [&](int it) {
    T* dst = Ks + (a.two_buffers ? (it & 1) * buffer : 0) + my_row * ldk;
    if (a.vec) {
#pragma unroll
      for (int k = 0; k < KI; ++k) {
        const int unit = my_unit + k * TPR;
        if (unit < 2 * steps) *reinterpret_cast<uint4*>(dst + unit * E) = reg[k];
      }
    } else {
      const T* src = static_cast<const T*>(a.rows) + static_cast<size_t>(max(reg_slot, 0)) * a.dk;
      for (int e = my_unit; e < 2 * E * steps; e += TPR) dst[e] = reg_slot >= 0 && e < a.dk ? src[e] : from_float<T>(0.f);
    }
  };

  f32x16 o[NVT];
#pragma unroll
  for (int dt = 0; dt < NVT; ++dt)
#pragma unroll
    for (int i = 0; i < 16; ++i) o[dt][i] = 0.f;
  float m = -INFINITY, l = 0.f;

  if (tid < kKeys) {
    slot_s[0][tid] = slot_of(chunk0 * kKeys + tid);
    slot_s[1][tid] = slot_of((chunk0 + 1) * kKeys + tid);
  }
  __syncthreads();
  ask(0);
  stash(0);
  __syncthreads();
  for (int it = 0; it < n_chunks; ++it) {
    const int key0 = (chunk0 + it) * kKeys;
    const T* K = Ks + (a.two_buffers ? (it & 1) * buffer : 0);
    if (it + 1 < n_chunks) ask(it + 1);
    if (tid < kKeys && it + 2 < n_chunks) slot_s[(it + 2) % kRing][tid] = slot_of(key0 + 2 * kKeys + tid);

    f32x16 s;
#pragma unroll
    for (int i = 0; i < 16; ++i) s[i] = 0.f;
    if (active) {
      // four steps' keys at a time, in two chains of sums; steps behind the row's last one meet a query of zeros
      const T* krow = K + c * ldk + E * h;
      f32x16 s2;
#pragma unroll
      for (int i = 0; i < 16; ++i) s2[i] = 0.f;
#pragma unroll
      for (int st0 = 0; st0 < KQ; st0 += 4) {
        if (st0 * SL + sl >= steps) continue;
        uint4 k4[4];
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (st0 + u < KQ) k4[u] = *reinterpret_cast<const uint4*>(krow + 2 * E * min((st0 + u) * SL + sl, steps - 1));
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (st0 + u < KQ) {
            f32x16& sum = u & 1 ? s2 : s;
            if constexpr (sizeof(T) == 2) {
              sum = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, k4[u]), __builtin_bit_cast(bf16x8, qf[st0 + u]), sum, 0, 0, 0);
            } else {
              const f32x4 kf = __builtin_bit_cast(f32x4, k4[u]), qq = __builtin_bit_cast(f32x4, qf[st0 + u]);
#pragma unroll
              for (int v = 0; v < 4; ++v) sum = __builtin_amdgcn_mfma_f32_32x32x2f32(kf[v], qq[v], sum, 0, 0, 0);
            }
          }
      }
#pragma unroll
      for (int i = 0; i < 16; ++i) s[i] += s2[i];
      if (SL > 1) {
        float* mine = sred + wave * 1024 + 4 * lane;
#pragma unroll
        for (int j = 0; j < 4; ++j) *reinterpret_cast<f32x4*>(mine + 256 * j) = f32x4{s[4 * j], s[4 * j + 1], s[4 * j + 2], s[4 * j + 3]};
      }
    }
    // Element i of s: key key0 + 8 (i / 4) + 4 h + i % 4, query c. Of SL waves each turns 16 / SL of them into weights:
    // the parts of its own ones are added up (in order), the maxima and then the weights go round through LDS.
    constexpr int EW = 16 / SL;
    if (SL > 1) lds_barrier();
    float w[EW], mx = -INFINITY;
    if (active) {
      if (SL > 1) {
        const float* base = sred + g * SL * 1024 + 4 * lane + 256 * (EW / 4) * sl;
#pragma unroll
        for (int j = 0; j < EW / 4; ++j) {
          f32x4 t = *reinterpret_cast<const f32x4*>(base + 256 * j);
#pragma unroll
          for (int o2 = 1; o2 < SL; ++o2) t += *reinterpret_cast<const f32x4*>(base + 1024 * o2 + 256 * j);
#pragma unroll
          for (int u = 0; u < 4; ++u) w[4 * j + u] = t[u];
        }
      } else {
#pragma unroll
        for (int i = 0; i < EW; ++i) w[i] = s[i];
      }
      if (key0 >= lo_last && key0 + kKeys - 1 <= pos0) {
#pragma unroll
        for (int i = 0; i < EW; ++i) w[i] *= a.scale2, mx = fmaxf(mx, w[i]);
      } else {
        const unsigned seen = static_cast<unsigned>(hi - lo), first = static_cast<unsigned>(key0 + 8 * (EW / 4) * sl + 4 * h - lo);
#pragma unroll
        for (int i = 0; i < EW; ++i) {
          w[i] = first + 8 * (i >> 2) + (i & 3) <= seen ? w[i] * a.scale2 : -INFINITY;
          mx = fmaxf(mx, w[i]);
        }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (SL > 1 && h == 0) row_s[wave][c] = mx;
    }
    if (SL > 1) lds_barrier();
    float alpha = 1.f;
    uint4 pieces[3][2];
    if (active) {
      if (SL > 1)
#pragma unroll
        for (int o2 = 0; o2 < SL; ++o2) mx = fmaxf(mx, row_s[g * SL + o2][c]);
      const float m_new = fmaxf(m, mx), m_use = m_new == -INFINITY ? 0.f : m_new;
      alpha = exp2_hw(m - m_use);
      m = m_new;
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < EW; ++i) w[i] = exp2_hw(w[i] - m_use), sum += w[i];
      l = l * alpha + sum;
      if constexpr (sizeof(T) == 2) {
        // piece pc of keys 16 b .. 16 b + 15: the lane's eight are those of elements 8 b .. 8 b + 7
        uint32_t w1[EW / 2], w2[EW / 2], w3[EW / 2];
#pragma unroll
        for (int u = 0; u < EW / 2; ++u) split_pair(w[2 * u], w[2 * u + 1], w1[u], w2[u], w3[u]);
        if constexpr (SL == 1) {
#pragma unroll
          for (int b = 0; b < 2; ++b) {
            pieces[0][b] = uint4{w1[4 * b], w1[4 * b + 1], w1[4 * b + 2], w1[4 * b + 3]};
            pieces[1][b] = uint4{w2[4 * b], w2[4 * b + 1], w2[4 * b + 2], w2[4 * b + 3]};
            pieces[2][b] = uint4{w3[4 * b], w3[4 * b + 1], w3[4 * b + 2], w3[4 * b + 3]};
          }
        } else {
#pragma unroll
          for (int j = 0; j < EW / 4; ++j) {
            const int quad = sl * (EW / 4) + j;  // elements 4 quad .. 4 quad + 3
            unsigned char* dst = Ps + g * weight_bytes<T>() + (quad >> 1) * 1024 + 16 * lane + 8 * (quad & 1);
            *reinterpret_cast<uint2*>(dst) = uint2{w1[2 * j], w1[2 * j + 1]};
            *reinterpret_cast<uint2*>(dst + 2048) = uint2{w2[2 * j], w2[2 * j + 1]};
            *reinterpret_cast<uint2*>(dst + 4096) = uint2{w3[2 * j], w3[2 * j + 1]};
          }
        }
      } else if constexpr (SL > 1) {
#pragma unroll
        for (int j = 0; j < EW / 4; ++j)
          *reinterpret_cast<f32x4*>(Ps + g * weight_bytes<T>() + (sl * (EW / 4) + j) * 1024 + 16 * lane) = f32x4{w[4 * j], w[4 * j + 1], w[4 * j + 2], w[4 * j + 3]};
      }
    }
    if (SL > 1) {
      // the other buffer's last readers, of the chunk before, have passed this chunk's first barrier
      if (a.two_buffers && it + 1 < n_chunks) stash(it + 1);
      lds_barrier();
    }
    if (active) {
      if (__ballot(alpha != 1.f))
#pragma unroll
        for (int dt = 0; dt < NVT; ++dt)
#pragma unroll
          for (int i = 0; i < 16; ++i) o[dt][i] *= alpha;
      if constexpr (sizeof(T) == 2) {
        const int j16 = lane & 15, col16 = 16 * ((lane >> 4) & 1);
#pragma unroll
        for (int b = 0; b < 2; ++b) {  // keys 16 b .. 16 b + 15; the lane's eight are 16 b + 4 h + u and 16 b + 8 + 4 h + u
          if constexpr (SL > 1)
#pragma unroll
            for (int pc = 0; pc < 3; ++pc) pieces[pc][b] = *reinterpret_cast<const uint4*>(Ps + g * weight_bytes<T>() + pc * 2048 + b * 1024 + 16 * lane);
          const bf16* vrow = reinterpret_cast<const bf16*>(K) + (16 * b + 4 * h + (j16 >> 2)) * ldk + col16 + 4 * (j16 & 3);
          // all columns' values first, then the pieces in turn, the smallest first: neighbouring products add to
          // different sums (columns behind the last tile repeat it, and nobody reads their sums)
          bf16x8 v8[NVT];
#pragma unroll
          for (int dt = 0; dt < NVT; ++dt) {
            const int d0 = 32 * min(sl * NVT + dt, last_tile);
            const uint2 v0 = read_transposed(vrow + d0), v1 = read_transposed(vrow + 8 * ldk + d0);
            v8[dt] = __builtin_bit_cast(bf16x8, uint4{v0.x, v0.y, v1.x, v1.y});
          }
#pragma unroll
          for (int pc = 2; pc >= 0; --pc)
#pragma unroll
            for (int dt = 0; dt < NVT; ++dt)
              o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v8[dt], __builtin_bit_cast(bf16x8, pieces[pc][b]), o[dt], 0, 0, 0);
        }
      } else {
        const float* v = reinterpret_cast<const float*>(K) + 4 * h * ldk + c;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          f32x4 p4;
          if constexpr (SL > 1) p4 = *reinterpret_cast<const f32x4*>(Ps + g * weight_bytes<T>() + j * 1024 + 16 * lane);
          else p4 = f32x4{w[4 * j], w[4 * j + 1], w[4 * j + 2], w[4 * j + 3]};
          float vv[4][NVT];
#pragma unroll
          for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int dt = 0; dt < NVT; ++dt) vv[u][dt] = v[(8 * j + u) * ldk + 32 * min(sl * NVT + dt, last_tile)];
#pragma unroll
          for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int dt = 0; dt < NVT; ++dt) o[dt] = __builtin_amdgcn_mfma_f32_32x32x2f32(vv[u][dt], p4[u], o[dt], 0, 0, 0);
        }
      }
    }
    if (SL == 1 || !a.two_buffers) {
      if (!a.two_buffers) lds_barrier();  // every wave is done with the one buffer
      if (it + 1 < n_chunks) stash(it + 1);
      lds_barrier();
    }
  }

  l += __shfl_xor(l, 32, 64);
  if (SL > 1) {  // the waves' shares of the weights, in order
    lds_barrier();
    if (h == 0) row_s[wave][c] = l;
    lds_barrier();
    l = 0.f;
#pragma unroll
    for (int o2 = 0; o2 < SL; ++o2) l += row_s[g * SL + o2][c];
  }
  if (!live) return;
  if (SINGLE && a.part) {
    const size_t at = (static_cast<size_t>(blockIdx.x) * a.heads + head) * a.spans + blockIdx.z;
    float* dst = a.part + at * a.rank;
#pragma unroll
    for (int dt = 0; dt < NVT; ++dt)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = 32 * (sl * NVT + dt) + 8 * j + 4 * h;
        if (a.rank % 4 == 0) {
          if (d < a.rank) *reinterpret_cast<f32x4*>(dst + d) = f32x4{o[dt][4 * j], o[dt][4 * j + 1], o[dt][4 * j + 2], o[dt][4 * j + 3]};
        } else {
#pragma unroll
          for (int u = 0; u < 4; ++u)
            if (d + u < a.rank) dst[d + u] = o[dt][4 * j + u];
        }
      }
    if (sl == 0 && h == 0) a.part_ml[2 * at] = m, a.part_ml[2 * at + 1] = l;
    return;
  }
  const float f = latent_factor(m, l, a.sink, head);
  T* dst = static_cast<T*>(a.out) + (static_cast<size_t>(token) * a.heads + head) * a.rank;
#pragma unroll
  for (int dt = 0; dt < NVT; ++dt)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int d = 32 * (sl * NVT + dt) + 8 * j + 4 * h;
      if (a.vec && d + 3 < a.rank) {
        Vec4<T>::store(dst + d, float4{o[dt][4 * j] * f, o[dt][4 * j + 1] * f, o[dt][4 * j + 2] * f, o[dt][4 * j + 3] * f});
      } else {
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (d + u < a.rank) dst[d + u] = from_float<T>(o[dt][4 * j + u] * f);
      }
    }
}

// The spans of a single token joined, in their order, with the sink: a block per token and head. The spans' factors are
// formed once, into LDS, up to kJoin of them at a time; W elements a thread, eight spans' sums asked for together.
constexpr int kJoin = 256;
template <typename T, int W>
__global__ __launch_bounds__(kJoin) void latent_join_kernel(const LatentArgs a) {
  __shared__ float scratch[16], factor_s[kJoin];
  const int n = a.list ? a.list[blockIdx.x] : blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
  const int pos = a.positions[n], lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int count = min(a.spans, pos / a.span - lo / a.span + 1);
  const size_t at = (static_cast<size_t>(blockIdx.x) * a.heads + head) * a.spans;
  const float* ml = a.part_ml + 2 * at;
  const float sink = a.sink ? a.sink[head] * kLog2e : -INFINITY;
  float M = sink;
  for (int s = tid; s < count; s += kJoin) M = fmaxf(M, ml[2 * s]);
  M = block_max(M, scratch);
  const float m_use = M == -INFINITY ? 0.f : M;
  float total[W], l = 0.f;
  const int d = W * tid;
  static_assert(W * kJoin >= 512, "a thread has all its elements at once");
#pragma unroll
  for (int e = 0; e < W; ++e) total[e] = 0.f;
  for (int s0 = 0; s0 < count; s0 += kJoin) {
    const int here = min(kJoin, count - s0);
    __syncthreads();
    float w = 0.f;
    if (tid < here) {
      w = exp2_hw(ml[2 * (s0 + tid)] - m_use);
      l = fmaf(ml[2 * (s0 + tid) + 1], w, l);
    }
    factor_s[tid] = w;
    __syncthreads();
    if (d < a.rank) {
      const float* src = a.part + (at + s0) * a.rank + d;
      for (int s = 0; s < here; s += 8) {
        float v[8][W];
#pragma unroll
        for (int u = 0; u < 8; ++u)
#pragma unroll
          for (int e = 0; e < W; ++e) v[u][e] = s + u < here && d + e < a.rank ? src[static_cast<size_t>(s + u) * a.rank + e] : 0.f;
#pragma unroll
        for (int u = 0; u < 8; ++u)
#pragma unroll
          for (int e = 0; e < W; ++e) total[e] = fmaf(v[u][e], factor_s[min(s + u, kJoin - 1)], total[e]);
      }
    }
  }
  l = block_sum(l, scratch);
  if (a.sink) l += exp2_hw(sink - m_use);
  if (d >= a.rank) return;
  T* dst = static_cast<T*>(a.out) + (static_cast<size_t>(n) * a.heads + head) * a.rank + d;
  const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
  for (int e = 0; e < W; ++e)
    if (d + e < a.rank) dst[e] = from_float<T>(total[e] * inv);
}

constexpr int kMaxRank = 512, kMaxRow = 640;

int check_args(const char* what, const LatentArgs& a, int dt, int n) {
  PYRE_REQUIRE(known_dtype(dt) && a.q && a.rows && a.out && a.positions && a.seq_of_token && a.table, "%s: bad arguments", what);
  PYRE_REQUIRE(a.rank > 0 && a.rank <= kMaxRank && a.dk >= a.rank && a.dk <= kMaxRow, "%s: rows of %d elements, %d of them values, are outside %d / %d",
               what, a.dk, a.rank, kMaxRow, kMaxRank);
  PYRE_REQUIRE(a.heads > 0 && a.heads <= 65535 && a.page_size > 0 && a.table_stride > 0 && a.window >= 0 && n >= 0, "%s: bad geometry", what);
  return 0;
}

// Launches one form; LDS is what the block asks for, raised once per form where it exceeds what a launch has by default.
template <typename T, int G, int SL, int NVT, int KQ, bool SINGLE>
int launch(const char* what, LatentArgs a, int blocks, int spans, hipStream_t stream) {
  constexpr int E = 16 / sizeof(T);
  const int steps = (a.dk + 2 * E - 1) / (2 * E), ldk = 2 * E * steps + E;
  PYRE_REQUIRE(steps <= KQ * SL && a.rank <= 32 * NVT * SL, "%s: rows of %d / %d elements do not fit the form", what, a.dk, a.rank);
  const size_t slack = 32 * NVT * SL > ldk ? 32 * NVT * SL - ldk : 0, exchange = SL > 1 ? sizeof(float) * G * SL * 1024 + G * weight_bytes<T>() : 0;
  auto k_bytes = [&](int buffers) { return sizeof(T) * ((buffers * kKeys * static_cast<size_t>(ldk) + slack + 7) / 8 * 8); };
  const size_t budget = 156 * 1024;
  a.two_buffers = k_bytes(2) + exchange <= budget - 16 * 1024 ? 1 : 0;
  size_t lds = k_bytes(a.two_buffers ? 2 : 1) + exchange;
  // the block's part of the request's block table, if it is not too long
  const int seen = a.window > 0 ? a.window + kKeys : a.table_stride * a.page_size;
  const int entries = min(seen / a.page_size + 2, a.table_stride + 1);
  a.tab_lds = lds + sizeof(int) * entries <= budget && entries <= 4096 ? entries : 0;
  lds += sizeof(int) * a.tab_lds;
  PYRE_REQUIRE(lds <= budget, "%s: %zu bytes of LDS are more than a block has", what, lds);
  const int groups = SINGLE ? (a.heads + 32 * G - 1) / (32 * G) : (a.heads + G - 1) / G;
  const auto kernel = &latent_attn_kernel<T, G, SL, NVT, KQ, SINGLE>;
  static size_t raised = 64 * 1024;
  if (lds > raised) {
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds)) != hipSuccess)
      return fail("%s: the device refuses %zu bytes of LDS", what, lds);
    raised = lds;
  }
  // prompt tiles come with those that see the most keys first: all heads of the longest start before the shorter ones,
  // which then fill the compute units that are done
  PYRE_REQUIRE(SINGLE || blocks <= 65535, "%s: %d tiles are more than a launch holds", what, blocks);
  const dim3 grid = SINGLE ? dim3(blocks, groups, spans) : dim3(groups, blocks, 1);
  hipLaunchKernelGGL((latent_attn_kernel<T, G, SL, NVT, KQ, SINGLE>), grid, dim3(64 * G * SL), lds, stream, a);
  return check_launch(what);
}

bool aligned_rows(const LatentArgs& a, int dt) {
  const int E = dt == kBF16 ? 8 : 4;
  return a.dk % E == 0 && a.rank % 4 == 0 && reinterpret_cast<uintptr_t>(a.q) % 16 == 0 && reinterpret_cast<uintptr_t>(a.rows) % 16 == 0 &&
         reinterpret_cast<uintptr_t>(a.out) % 16 == 0;
}

}  // namespace

extern "C" int pyre_latent_attn_tile(const void* q, const void* rows, void* out, int dt, const int* tiles, int n_tiles,
                                     const int* positions, const int* seq_of_token, const int* block_table, int table_stride,
                                     int heads, int rank, int dk, int page_size, float scale, int window, const float* sink,
                                     hipStream_t stream) {
  LatentArgs a{};
  a.q = q, a.rows = rows, a.out = out, a.list = tiles, a.positions = positions, a.seq_of_token = seq_of_token, a.table = block_table;
  a.sink = sink, a.table_stride = table_stride, a.heads = heads, a.rank = rank, a.dk = dk, a.page_size = page_size, a.window = window;
  a.scale2 = scale * kLog2e;
  if (check_args("latent_attn_tile", a, dt, n_tiles)) return 1;
  if (n_tiles == 0) return 0;
  PYRE_REQUIRE(tiles, "latent_attn_tile: no tiles");
  a.vec = aligned_rows(a, dt);
  // waves that share a row tile: as few as hold the row and the output in their registers
  if (rank <= 128 && dk <= 128 && dt == kBF16) return launch<bf16, 4, 1, 4, 8, false>("latent_attn_tile", a, n_tiles, 1, stream);
  if (rank <= 128 && dk <= 256)
    return dt == kBF16 ? launch<bf16, 4, 1, 4, 16, false>("latent_attn_tile", a, n_tiles, 1, stream)
                       : launch<float, 4, 1, 4, 32, false>("latent_attn_tile", a, n_tiles, 1, stream);
  if (rank <= 256 && dk <= 384)
    return dt == kBF16 ? launch<bf16, 4, 2, 4, 12, false>("latent_attn_tile", a, n_tiles, 1, stream)
                       : launch<float, 2, 2, 4, 24, false>("latent_attn_tile", a, n_tiles, 1, stream);
  return dt == kBF16 ? launch<bf16, 2, 4, 4, 10, false>("latent_attn_tile", a, n_tiles, 1, stream)
                     : launch<float, 1, 4, 4, 20, false>("latent_attn_tile", a, n_tiles, 1, stream);
}

// Spans that a single token's keys are dealt to: one where the window is short, else of 64 keys (256 without a window
// or behind a very long one). The number follows from the window and the widest context of the launch, the span's size
// from the window alone.
static int span_of(int window) { return window > 0 && window <= 256 ? 0 : window > 0 && window <= 4096 ? 64 : 256; }

extern "C" int pyre_latent_attn_spans(int max_keys, int window) {
  const int span = span_of(window);
  if (span == 0) return 1;
  const int seen = window > 0 && window < max_keys ? window : max_keys;
  return (seen > 0 ? seen - 1 : 0) / span + 2;  // a window that starts inside a span touches one more
}

extern "C" int pyre_latent_attn_single(const void* q, const void* rows, void* out, int dt, const int* tokens, int n,
                                       const int* positions, const int* seq_of_token, const int* block_table, int table_stride,
                                       int heads, int rank, int dk, int page_size, float scale, int window, const float* sink,
                                       float* part, hipStream_t stream) {
  LatentArgs a{};
  a.q = q, a.rows = rows, a.out = out, a.list = tokens, a.positions = positions, a.seq_of_token = seq_of_token, a.table = block_table;
  a.sink = sink, a.table_stride = table_stride, a.heads = heads, a.rank = rank, a.dk = dk, a.page_size = page_size, a.window = window;
  a.scale2 = scale * kLog2e;
  if (check_args("latent_attn_single", a, dt, n)) return 1;
  if (n == 0) return 0;
  a.vec = aligned_rows(a, dt);
  a.span = span_of(window);
  a.spans = pyre_latent_attn_spans(table_stride * page_size, window);
  PYRE_REQUIRE(a.spans == 1 || (part && reinterpret_cast<uintptr_t>(part) % 16 == 0), "latent_attn_single: %d spans need scratch", a.spans);
  PYRE_REQUIRE(a.spans <= 65535, "latent_attn_single: %d spans are not a launch", a.spans);
  a.part = a.span ? part : nullptr;
  a.part_ml = a.part ? part + static_cast<size_t>(n) * heads * a.spans * rank : nullptr;
  if (a.span == 0) a.spans = 1;
  int bad;
  if (rank <= 128)
    bad = dt == kBF16 ? launch<bf16, 1, 4, 1, 10, true>("latent_attn_single", a, n, a.spans, stream)
                      : launch<float, 1, 4, 1, 20, true>("latent_attn_single", a, n, a.spans, stream);
  else if (rank <= 256)
    bad = dt == kBF16 ? launch<bf16, 1, 4, 2, 10, true>("latent_attn_single", a, n, a.spans, stream)
                      : launch<float, 1, 4, 2, 20, true>("latent_attn_single", a, n, a.spans, stream);
  else
    bad = dt == kBF16 ? launch<bf16, 1, 4, 4, 10, true>("latent_attn_single", a, n, a.spans, stream)
                      : launch<float, 1, 4, 4, 20, true>("latent_attn_single", a, n, a.spans, stream);
  if (bad) return bad;
  if (a.part)
    PYRE_DISPATCH(dt, T, hipLaunchKernelGGL((latent_join_kernel<T, 2>), dim3(n, heads), dim3(kJoin), 0, stream, a));
  return check_launch("latent_attn_single");
}
