// What stands between the input product and the attention kernels of two mixers that keep less than a
// key and a value per head and token, and the small per-head products of the second:
//
//   rope_tied_write  attention whose values are its keys as projected: sums the product's partial sums,
//                    adds the bias, turns the first `rot` elements of every query and key head by position
//                    (element e with e + rot/2), stores the queries, the turned keys as keys and the keys
//                    as they were before turning as values (k, v [pages, nkv, page, d]).
//   latent_rows      attention over one compressed row per token: what an input product holds for it. Queries, either
//                    split into their unturned part (rows) and their turned part (turned by position, straight into the
//                    wide queries that the attention kernels read), or a compressed row of queries, divided by its root
//                    mean square, times a gain; the token's row [c | r]: c divided by its root mean square, times a
//                    gain, r turned by position, into its page; the sigmoids of a gate.
//   head_matmul      out[n, h, :] = W[h] x[n, h, :] (times a gate) for every head h, W [heads, dout, din]: the products
//                    that carry a query into the compressed row's space and a weighted row out of it.
//
// All arithmetic is float32; roundings happen at the stores of 16-bit outputs only.
#include "pyre_api.h"
#include "pyre_common.h"
#include "pyre_vec4.h"

using namespace pyre;

namespace {

constexpr int kThreads = 256;

struct Proj {
  const void* data;
  int dt, count;
  size_t stride;
  int ld, col0;
  const void* bias;
  int bias_dt;
};

__device__ inline float proj_at(const Proj& p, int n, int col) {
  const size_t at = static_cast<size_t>(n) * p.ld + p.col0 + col;
  float v = 0.f;
  for (int i = 0; i < p.count; ++i) v += load_as_float(p.data, p.dt, i * p.stride + at);
  if (p.bias) v += load_as_float(p.bias, p.bias_dt, col);
  return v;
}

template <typename TC>
__global__ __launch_bounds__(kThreads) void rope_tied_write_kernel(Proj proj, void* __restrict__ q_out, int q_dt,
                                                                   TC* __restrict__ k_cache, TC* __restrict__ v_cache,
                                                                   const float* __restrict__ cos_t,
                                                                   const float* __restrict__ sin_t, int rot,
                                                                   const int* __restrict__ positions,
                                                                   const int* __restrict__ slots, int nq, int nkv, int d,
                                                                   int page_size, int write_kv) {
  const int n = blockIdx.x, half = rot / 2;
  const int pos = positions[n];
  const int slot = write_kv ? slots[n] : -1;
  const int page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
  for (int i = threadIdx.x; i < (nq + nkv) * d; i += kThreads) {
    const int head = i / d, e = i % d;
    const float x = proj_at(proj, n, i);
    float turned = x;
    if (e < rot) {
      const int j = e < half ? e : e - half;
      const float c = cos_t[static_cast<size_t>(pos) * half + j], s = sin_t[static_cast<size_t>(pos) * half + j];
      const float y = proj_at(proj, n, head * d + (e < half ? e + half : e - half));
      float a, b;
      if (e < half) {
        rotate_pair(x, y, c, s, a, b);
        turned = a;
      } else {
        rotate_pair(y, x, c, s, a, b);
        turned = b;
      }
    }
    if (head < nq) {
      store_from_float(q_out, q_dt, static_cast<size_t>(n) * nq * d + i, turned);
    } else if (slot >= 0) {
      const size_t at = ((static_cast<size_t>(page) * nkv + (head - nq)) * page_size + off) * d + e;
      k_cache[at] = from_float<TC>(turned);
      v_cache[at] = from_float<TC>(x);
    }
  }
}

// The same with a wave per token and head, four elements a lane and an element's partial sums asked for together:
// head sizes, the number of turned elements of each half, the product's width, first column and stride are multiples
// of four; queries, caches and bias share one element type.
template <typename TP, typename TC>
__global__ __launch_bounds__(kWave) void rope_tied_write_vec_kernel(const TP* __restrict__ proj, int count, size_t stride,
                                                                    int ld, int col0, const TC* __restrict__ bias,
                                                                    TC* __restrict__ q_out, TC* __restrict__ k_cache,
                                                                    TC* __restrict__ v_cache, const float* __restrict__ cos_t,
                                                                    const float* __restrict__ sin_t, int rot,
                                                                    const int* __restrict__ positions,
                                                                    const int* __restrict__ slots, int nq, int nkv, int d,
                                                                    int page_size, int write_kv) {
  __shared__ __attribute__((aligned(16))) float xs[4 * kWave];
  const int n = blockIdx.x, head = blockIdx.y, e = 4 * threadIdx.x, half = rot / 2;
  float4 x = {0.f, 0.f, 0.f, 0.f};
  if (e < d) {
    x = sum_partials4(proj + static_cast<size_t>(n) * ld + col0 + head * d + e, stride, count);
    if (bias) x = add4(x, Vec4<TC>::load(bias + head * d + e));
    *reinterpret_cast<float4*>(xs + e) = x;
  }
  __syncthreads();
  if (e >= d) return;
  float4 t = x;
  if (e < rot) {  // the four elements lie in the same half, their partners in the other
    const bool low = e < half;
    const int j = low ? e : e - half;
    const float4 y = *reinterpret_cast<const float4*>(xs + (low ? e + half : e - half));
    const size_t at = static_cast<size_t>(positions[n]) * half + j;
    const float4 c = *reinterpret_cast<const float4*>(cos_t + at), sn = *reinterpret_cast<const float4*>(sin_t + at);
    float a, b;
    if (low) {
      rotate_pair(x.x, y.x, c.x, sn.x, a, b), t.x = a;
      rotate_pair(x.y, y.y, c.y, sn.y, a, b), t.y = a;
      rotate_pair(x.z, y.z, c.z, sn.z, a, b), t.z = a;
      rotate_pair(x.w, y.w, c.w, sn.w, a, b), t.w = a;
    } else {
      rotate_pair(y.x, x.x, c.x, sn.x, a, b), t.x = b;
      rotate_pair(y.y, x.y, c.y, sn.y, a, b), t.y = b;
      rotate_pair(y.z, x.z, c.z, sn.z, a, b), t.z = b;
      rotate_pair(y.w, x.w, c.w, sn.w, a, b), t.w = b;
    }
  }
  if (head < nq) {
    Vec4<TC>::store(q_out + (static_cast<size_t>(n) * nq + head) * d + e, t);
    return;
  }
  const int slot = write_kv ? slots[n] : -1;
  if (slot < 0) return;
  const size_t at = ((static_cast<size_t>(slot / page_size) * nkv + (head - nq)) * page_size + slot % page_size) * d + e;
  Vec4<TC>::store(k_cache + at, t);
  Vec4<TC>::store(v_cache + at, x);
}

// One product's columns for attention over a compressed row, any of the parts present. A token's blocks: one for the
// row, one for the compressed queries, then blocks of kThreads * W columns for the split queries and for the gate.
// W = 4: four columns a thread (sizes, first columns, strides and turned halves are multiples of four).
struct LatentRows {
  const void* proj;
  size_t stride;
  int count, ld;
  const float* cos_t;
  const float* sin_t;
  const int* positions;
  // split queries: heads of [dim | rot] at column q0; q_out [n][heads * dim], turned parts to wide [n][heads][rank + rot]
  int heads, dim, q0;
  void* q_out;
  void* wide;
  // compressed queries: q_rank columns at q0, normed into q_out [n][q_rank]
  int q_rank;
  const float* q_gain;
  // the row: rank + rot columns at r0, into cache [pages][1][page][rank + rot] at slots
  int rank, rot, neighbours, r0;
  void* cache;
  const float* gain;
  const int* slots;
  // the gate: gate_width columns at g0, float32 [n][gate_width]
  int gate_width, g0;
  float* gate;
  float eps;
  int row_blocks, norm_blocks, query_blocks;
};

template <typename TP, int W>
__device__ inline void columns(const LatentRows& a, int n, int col, float (&v)[W]) {
  const TP* src = static_cast<const TP*>(a.proj) + static_cast<size_t>(n) * a.ld + col;
  if constexpr (W == 4) {
    const float4 x = sum_partials4(src, a.stride, a.count);
    v[0] = x.x, v[1] = x.y, v[2] = x.z, v[3] = x.w;
  } else {
    v[0] = 0.f;
    for (int p = 0; p < a.count; ++p) v[0] += to_float(src[p * a.stride]);
  }
}

template <typename T, int W>
__device__ inline void put(T* dst, const float (&v)[W]) {
  if constexpr (W == 4) Vec4<T>::store(dst, float4{v[0], v[1], v[2], v[3]});
  else *dst = from_float<T>(v[0]);
}

// Elements e .. e + W - 1 of a part of `rot` turned elements that starts at column col, turned.
template <typename TP, int W>
__device__ inline void turned(const LatentRows& a, int n, int col, int e, float (&out)[W]) {
  const int half = a.rot / 2;
  const size_t at = static_cast<size_t>(a.positions[n]) * half;
  float x[W], lost;
  columns<TP, W>(a, n, col + e, x);
  if (!a.neighbours) {  // element j with j + half; the W elements lie in one half
    const bool low = e < half;
    const int j = low ? e : e - half;
    float y[W];
    columns<TP, W>(a, n, col + (low ? e + half : e - half), y);
#pragma unroll
    for (int u = 0; u < W; ++u) {
      const float c = a.cos_t[at + j + u], s = a.sin_t[at + j + u];
      if (low) rotate_pair(x[u], y[u], c, s, out[u], lost);
      else rotate_pair(y[u], x[u], c, s, lost, out[u]);
    }
  } else if constexpr (W == 4) {
#pragma unroll
    for (int u = 0; u < W; u += 2) rotate_pair(x[u], x[u + 1], a.cos_t[at + (e + u) / 2], a.sin_t[at + (e + u) / 2], out[u], out[u + 1]);
  } else {
    float y[W];
    columns<TP, W>(a, n, col + (e ^ 1), y);
    const float c = a.cos_t[at + e / 2], s = a.sin_t[at + e / 2];
    if (e & 1) rotate_pair(y[0], x[0], c, s, lost, out[0]);
    else rotate_pair(x[0], y[0], c, s, out[0], lost);
  }
}

template <typename TP, typename T, int W>
__global__ __launch_bounds__(kThreads) void latent_rows_kernel(const LatentRows a) {
  __shared__ float scratch[16];
  const int n = blockIdx.x, tid = threadIdx.x;
  int b = blockIdx.y;
  if (b < a.row_blocks + a.norm_blocks) {  // a normed part: the row, or the compressed queries
    const bool row = b < a.row_blocks;
    const int width = row ? a.rank : a.q_rank, col = row ? a.r0 : a.q0;
    const float* gain = row ? a.gain : a.q_gain;
    const int slot = row ? a.slots[n] : 0;
    T* dst = row ? static_cast<T*>(a.cache) + static_cast<size_t>(max(slot, 0)) * (a.rank + a.rot)
                 : static_cast<T*>(a.q_out) + static_cast<size_t>(n) * a.q_rank;
    float first[W], ss = 0.f;  // the thread's first columns stay in registers; wider parts are summed again below
    for (int i = W * tid; i < width; i += W * kThreads) {
      float v[W];
      columns<TP, W>(a, n, col + i, v);
#pragma unroll
      for (int u = 0; u < W; ++u) {
        ss += v[u] * v[u];
        if (i == W * tid) first[u] = v[u];
      }
    }
    ss = block_sum(ss, scratch);
    if (row && slot < 0) return;
    const float inv = 1.f / sqrtf(ss / static_cast<float>(width) + a.eps);
    for (int i = W * tid; i < width; i += W * kThreads) {
      float v[W];
      if (i == W * tid) {
#pragma unroll
        for (int u = 0; u < W; ++u) v[u] = first[u];
      } else {
        columns<TP, W>(a, n, col + i, v);
      }
#pragma unroll
      for (int u = 0; u < W; ++u) v[u] *= inv * gain[i + u];
      put<T, W>(dst + i, v);
    }
    if (row)
      for (int e = W * tid; e < a.rot; e += W * kThreads) {
        float v[W];
        turned<TP, W>(a, n, a.r0 + a.rank, e, v);
        put<T, W>(dst + a.rank + e, v);
      }
    return;
  }
  b -= a.row_blocks + a.norm_blocks;
  if (b < a.query_blocks) {
    const int per = a.dim + a.rot, i = W * (b * kThreads + tid);
    if (i >= a.heads * per) return;
    const int head = i / per, e = i % per;
    float v[W];
    if (e < a.dim) {
      columns<TP, W>(a, n, a.q0 + i, v);
      put<T, W>(static_cast<T*>(a.q_out) + (static_cast<size_t>(n) * a.heads + head) * a.dim + e, v);
    } else {
      turned<TP, W>(a, n, a.q0 + head * per + a.dim, e - a.dim, v);
      put<T, W>(static_cast<T*>(a.wide) + (static_cast<size_t>(n) * a.heads + head) * (a.rank + a.rot) + a.rank + (e - a.dim), v);
    }
    return;
  }
  b -= a.query_blocks;
  const int i = W * (b * kThreads + tid);
  if (i >= a.gate_width) return;
  float v[W];
  columns<TP, W>(a, n, a.g0 + i, v);
#pragma unroll
  for (int u = 0; u < W; ++u) v[u] = 1.f / (1.f + expf(-v[u]));
  put<float, W>(a.gate + static_cast<size_t>(n) * a.gate_width + i, v);
}

// ---------------------------------------------------------------------------------------------
typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef float f32x4 __attribute__((ext_vector_type(4)));

struct HeadProduct {
  const void* x;   // token n, head h at x + n * x_token + h * x_head
  const void* w;   // [heads][dout][din]
  void* out;
  const float* gate;  // [n][heads * dout] or null
  long x_token, x_head, out_token, out_head;
  int n, heads, din, dout;
};

template <typename T>
__device__ __forceinline__ f32x16 mfma_unit(uint4 a, uint4 b, f32x16 acc) {
  if constexpr (sizeof(T) == 2) {
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), acc, 0, 0, 0);
  } else {
    const f32x4 af = __builtin_bit_cast(f32x4, a), bf = __builtin_bit_cast(f32x4, b);
#pragma unroll
    for (int u = 0; u < 4; ++u) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(af[u], bf[u], acc, 0, 0, 0);
  }
  return acc;
}

template <typename T>
__device__ __forceinline__ void head_store(const HeadProduct& a, int token, int head, int h, int col0, const f32x16& acc) {
  if (token >= a.n) return;
  T* dst = static_cast<T*>(a.out) + token * a.out_token + head * a.out_head;
  const float* gate = a.gate ? a.gate + (static_cast<size_t>(token) * a.heads + head) * a.dout : nullptr;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int d = col0 + 8 * j + 4 * h;
    float v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) v[u] = d + u < a.dout ? acc[4 * j + u] * (gate ? gate[d + u] : 1.f) : 0.f;
    if (d + 3 < a.dout && reinterpret_cast<uintptr_t>(dst + d) % (4 * sizeof(T)) == 0) {
      Vec4<T>::store(dst + d, float4{v[0], v[1], v[2], v[3]});
    } else {
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (d + u < a.dout) dst[d + u] = from_float<T>(v[u]);
    }
  }
}

// On the matrix cores: rows of the tile are columns of the output (W's rows), its columns are tokens, so that a lane
// holds neighbouring outputs of one token. A lane's operands are 16-byte units of W's rows and of x, straight from
// memory (both are small and shared by many blocks). Few tokens: a block is one tile of 32 outputs and 32 tokens whose
// inner product its four waves share (parts added through LDS, in order).
template <typename T>
__global__ __launch_bounds__(kThreads) void head_matmul_few_kernel(const HeadProduct a) {
  constexpr int E = 16 / sizeof(T), kAhead = 8;
  __shared__ __attribute__((aligned(16))) float parts[3][4][64][4];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, h = lane >> 5, c = lane & 31;
  const int head = blockIdx.y, col0 = blockIdx.z * 32, token = blockIdx.x * 32 + c;
  const int steps = (a.din + 2 * E - 1) / (2 * E), per = (steps + 3) / 4, s0 = wave * per, s1 = min(steps, s0 + per);
  const T* wrow = static_cast<const T*>(a.w) + (static_cast<size_t>(head) * a.dout + min(col0 + c, a.dout - 1)) * a.din + E * h;
  const T* xrow = static_cast<const T*>(a.x) + min(token, a.n - 1) * a.x_token + head * a.x_head + E * h;
  f32x16 acc;
#pragma unroll
  for (int i = 0; i < 16; ++i) acc[i] = 0.f;
  for (int s = s0; s < s1; s += kAhead) {  // so many steps' operands on their way together
    uint4 wv[kAhead], xv[kAhead];
#pragma unroll
    for (int u = 0; u < kAhead; ++u) {
      const bool in = s + u < s1 && 2 * E * (s + u) + E * h < a.din;
      wv[u] = xv[u] = uint4{0u, 0u, 0u, 0u};
      if (!in) continue;
      wv[u] = *reinterpret_cast<const uint4*>(wrow + 2 * E * (s + u));
      xv[u] = *reinterpret_cast<const uint4*>(xrow + 2 * E * (s + u));
    }
#pragma unroll
    for (int u = 0; u < kAhead; ++u) acc = mfma_unit<T>(wv[u], xv[u], acc);
  }
  if (wave > 0)
#pragma unroll
    for (int j = 0; j < 4; ++j) *reinterpret_cast<f32x4*>(parts[wave - 1][j][lane]) = f32x4{acc[4 * j], acc[4 * j + 1], acc[4 * j + 2], acc[4 * j + 3]};
  __syncthreads();
  if (wave > 0) return;
#pragma unroll
  for (int w = 0; w < 3; ++w)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const f32x4 p = *reinterpret_cast<const f32x4*>(parts[w][j][lane]);
#pragma unroll
      for (int u = 0; u < 4; ++u) acc[4 * j + u] += p[u];
    }
  head_store<T>(a, token, head, h, col0, acc);
}

// Many tokens (bfloat16): a block has 128 outputs of a head against 128 tokens, a wave 64 x 64 of them; 64 elements of the
// inner product at a time through two buffers in LDS, the next ones on their way meanwhile. The results go out through
// LDS as well, so that a token's outputs are stored in whole lines (and its gate is read in such).
constexpr int kTile = 128, kSlice = 64, kSlicePad = kSlice + 8, kOutPad = kTile + 8;
__global__ __launch_bounds__(kThreads) void head_matmul_many_kernel(const HeadProduct a, int wide_stores) {
  __shared__ __attribute__((aligned(16))) bf16 lds[2 * 2 * kTile * kSlicePad];  // [buffer][W rows, tokens][kTile][kSlicePad]
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = lane >> 5, c = lane & 31;
  const int head = blockIdx.y, col0 = blockIdx.z * kTile, tok0 = blockIdx.x * kTile;
  const int slices = (a.din + kSlice - 1) / kSlice;
  // a thread brings 16 bytes of four W rows and of four tokens a slice: rows r, r + 32, ..., the same eight elements of each
  const int r = tid >> 3, e8 = 8 * (tid & 7);
  const bf16* w_src = static_cast<const bf16*>(a.w) + static_cast<size_t>(head) * a.dout * a.din + e8;
  const bf16* x_src = static_cast<const bf16*>(a.x) + head * a.x_head + e8;
  uint4 w_reg[4], x_reg[4];
  auto ask = [&](int s) {
    const bool in = s * kSlice + e8 < a.din;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      w_reg[k] = x_reg[k] = uint4{0u, 0u, 0u, 0u};
      if (!in) continue;
      w_reg[k] = *reinterpret_cast<const uint4*>(w_src + static_cast<size_t>(min(col0 + r + 32 * k, a.dout - 1)) * a.din + s * kSlice);
      x_reg[k] = *reinterpret_cast<const uint4*>(x_src + min(tok0 + r + 32 * k, a.n - 1) * a.x_token + s * kSlice);
    }
  };
  auto stash = [&](int s) {
    bf16* dst = lds + (s & 1) * 2 * kTile * kSlicePad + r * kSlicePad + e8;
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      *reinterpret_cast<uint4*>(dst + 32 * k * kSlicePad) = w_reg[k];
      *reinterpret_cast<uint4*>(dst + (kTile + 32 * k) * kSlicePad) = x_reg[k];
    }
  };
  f32x16 acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int u = 0; u < 16; ++u) acc[i][t][u] = 0.f;
  const int wr = 64 * (wave & 1), wt = 64 * (wave >> 1);
  ask(0);
  stash(0);
  __syncthreads();
  for (int s = 0; s < slices; ++s) {
    if (s + 1 < slices) ask(s + 1);
    const bf16* ws = lds + (s & 1) * 2 * kTile * kSlicePad + (wr + c) * kSlicePad + 8 * h;
    const bf16* xs = lds + (s & 1) * 2 * kTile * kSlicePad + (kTile + wt + c) * kSlicePad + 8 * h;
#pragma unroll
    for (int e = 0; e < kSlice; e += 16) {
      uint4 wv[2], xv[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        wv[i] = *reinterpret_cast<const uint4*>(ws + 32 * i * kSlicePad + e);
        xv[i] = *reinterpret_cast<const uint4*>(xs + 32 * i * kSlicePad + e);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int t = 0; t < 2; ++t) acc[i][t] = mfma_unit<bf16>(wv[i], xv[t], acc[i][t]);
    }
    if (s + 1 < slices) stash(s + 1);  // into the buffer whose readers passed the barrier before
    __syncthreads();
  }
  if (!wide_stores) {
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int i = 0; i < 2; ++i) head_store<bf16>(a, tok0 + wt + 32 * t + c, head, h, col0 + wr + 32 * i, acc[i][t]);
    return;
  }
  bf16* rows = lds;  // [kTile tokens][kOutPad]
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int t_in = wt + 32 * t + c, d_in = wr + 32 * i + 8 * j + 4 * h;
        float4 v = {acc[i][t][4 * j], acc[i][t][4 * j + 1], acc[i][t][4 * j + 2], acc[i][t][4 * j + 3]};
        if (a.gate && tok0 + t_in < a.n && col0 + d_in < a.dout) {
          const float4 gv = Vec4<float>::load(a.gate + (static_cast<size_t>(tok0 + t_in) * a.heads + head) * a.dout + col0 + d_in);
          v = float4{v.x * gv.x, v.y * gv.y, v.z * gv.z, v.w * gv.w};
        }
        Vec4<bf16>::store(rows + t_in * kOutPad + d_in, v);
      }
  __syncthreads();
  for (int k = tid; k < kTile * (kTile / 8); k += kThreads) {
    const int t = k / (kTile / 8), d = 8 * (k % (kTile / 8));
    if (tok0 + t < a.n && col0 + d < a.dout)
      *reinterpret_cast<uint4*>(static_cast<bf16*>(a.out) + (tok0 + t) * a.out_token + head * a.out_head + col0 + d) =
          *reinterpret_cast<const uint4*>(rows + t * kOutPad + d);
  }
}

// Any sizes: a thread an output.
template <typename T>
__global__ __launch_bounds__(kThreads) void head_matmul_any_kernel(const HeadProduct a) {
  const int n = blockIdx.x, head = blockIdx.y, d = blockIdx.z * kThreads + threadIdx.x;
  if (d >= a.dout) return;
  const T* x = static_cast<const T*>(a.x) + n * a.x_token + head * a.x_head;
  const T* w = static_cast<const T*>(a.w) + (static_cast<size_t>(head) * a.dout + d) * a.din;
  float v = 0.f;
  for (int e = 0; e < a.din; ++e) v = fmaf(to_float(w[e]), to_float(x[e]), v);
  if (a.gate) v *= a.gate[(static_cast<size_t>(n) * a.heads + head) * a.dout + d];
  static_cast<T*>(a.out)[n * a.out_token + head * a.out_head + d] = from_float<T>(v);
}

}  // namespace

extern "C" int pyre_rope_tied_write(const void* proj, int proj_dt, int n_partials, long partial_stride, int ld, int col0,
                                    const void* bias, int bias_dt, void* q_out, int q_dt, void* k_cache, void* v_cache,
                                    int cache_dt, const float* cos_t, const float* sin_t, int rot, const int* positions,
                                    const int* slots, int n, int nq, int nkv, int d, int page_size, int write_kv,
                                    hipStream_t stream) {
  PYRE_REQUIRE(known_dtype(proj_dt) && known_dtype(q_dt) && known_dtype(cache_dt) && n_partials >= 1, "rope_tied_write: bad dtypes");
  PYRE_REQUIRE(!bias || known_dtype(bias_dt), "rope_tied_write: unknown bias dtype");
  PYRE_REQUIRE(nq > 0 && nkv > 0 && d > 0 && page_size > 0, "rope_tied_write: bad geometry");
  PYRE_REQUIRE(rot >= 0 && rot <= d && rot % 2 == 0 && (rot == 0 || (cos_t && sin_t)), "rope_tied_write: %d turned elements do not fit a head of %d", rot, d);
  PYRE_REQUIRE(!write_kv || (k_cache && v_cache && slots), "rope_tied_write: a cache write needs caches and slots");
  if (n <= 0) return 0;
  const auto a16 = [](const void* q) { return reinterpret_cast<uintptr_t>(q) % 16 == 0; };
  if (d % 4 == 0 && d <= 4 * kWave && rot % 8 == 0 && ld % 4 == 0 && col0 % 4 == 0 && partial_stride % 4 == 0 && q_dt == cache_dt &&
      (!bias || bias_dt == cache_dt) && nq + nkv <= 65535 && a16(proj) && a16(bias) && a16(q_out) && a16(k_cache) && a16(v_cache) &&
      a16(cos_t) && a16(sin_t)) {
    PYRE_DISPATCH(proj_dt, TP, PYRE_DISPATCH(cache_dt, TC,
        hipLaunchKernelGGL((rope_tied_write_vec_kernel<TP, TC>), dim3(n, nq + nkv), dim3(kWave), 0, stream,
                           static_cast<const TP*>(proj), n_partials, static_cast<size_t>(partial_stride), ld, col0,
                           static_cast<const TC*>(bias), static_cast<TC*>(q_out), static_cast<TC*>(k_cache),
                           static_cast<TC*>(v_cache), cos_t, sin_t, rot, positions, slots, nq, nkv, d, page_size, write_kv)));
    return check_launch("rope_tied_write");
  }
  const Proj p{proj, proj_dt, n_partials, static_cast<size_t>(partial_stride), ld, col0, bias, bias_dt};
  PYRE_DISPATCH(cache_dt, TC,
      hipLaunchKernelGGL(rope_tied_write_kernel<TC>, dim3(n), dim3(kThreads), 0, stream, p, q_out, q_dt,
                         static_cast<TC*>(k_cache), static_cast<TC*>(v_cache), cos_t, sin_t, rot, positions, slots, nq,
                         nkv, d, page_size, write_kv));
  return check_launch("rope_tied_write");
}

extern "C" int pyre_latent_rows(const void* proj, int proj_dt, int n_partials, long partial_stride, int ld, int dt,
                                const float* cos_t, const float* sin_t, int neighbours, const int* positions, int rank, int rot,
                                int heads, int dim, int q_rank, int q0, void* q_out, void* wide, const float* q_gain,
                                int r0, void* cache, const float* gain, const int* slots, int gate_width, int g0,
                                float* gate, float eps, int n, hipStream_t stream) {
  PYRE_REQUIRE(known_dtype(proj_dt) && known_dtype(dt) && n_partials >= 1 && proj && ld > 0, "latent_rows: bad product");
  PYRE_REQUIRE(rank > 0 && rot >= 0 && rot % 2 == 0 && (rot == 0 || (cos_t && sin_t && positions)), "latent_rows: %d turned elements", rot);
  PYRE_REQUIRE(heads >= 0 && q_rank >= 0 && (heads == 0 || q_rank == 0) && (heads == 0 || (dim > 0 && q_out && (rot == 0 || wide))) &&
                   (q_rank == 0 || (q_gain && q_out)), "latent_rows: bad queries");
  PYRE_REQUIRE(!cache || (gain && slots), "latent_rows: a row needs a gain and slots");
  PYRE_REQUIRE(gate_width >= 0 && (gate_width == 0 || gate) && (eps > 0.f || (!cache && q_rank == 0)), "latent_rows: bad gate or eps");
  PYRE_REQUIRE((heads == 0 || (q0 >= 0 && q0 + heads * (dim + rot) <= ld)) && (q_rank == 0 || (q0 >= 0 && q0 + q_rank <= ld)) &&
                   (!cache || (r0 >= 0 && r0 + rank + rot <= ld)) && (gate_width == 0 || (g0 >= 0 && g0 + gate_width <= ld)),
               "latent_rows: columns outside the product's %d", ld);
  if (n <= 0) return 0;
  LatentRows a{};
  a.proj = proj, a.stride = static_cast<size_t>(partial_stride), a.count = n_partials, a.ld = ld;
  a.cos_t = cos_t, a.sin_t = sin_t, a.positions = positions, a.neighbours = neighbours;
  a.heads = heads, a.dim = dim, a.q0 = q0, a.q_out = q_out, a.wide = wide, a.q_rank = q_rank, a.q_gain = q_gain;
  a.rank = rank, a.rot = rot, a.r0 = r0, a.cache = cache, a.gain = gain, a.slots = slots;
  a.gate_width = gate_width, a.g0 = g0, a.gate = gate, a.eps = eps;
  a.row_blocks = cache ? 1 : 0, a.norm_blocks = q_rank > 0 ? 1 : 0;
  const auto a16 = [](const void* q) { return reinterpret_cast<uintptr_t>(q) % 16 == 0; };
  const bool vec = ld % 4 == 0 && partial_stride % 4 == 0 && q0 % 4 == 0 && r0 % 4 == 0 && g0 % 4 == 0 && rank % 4 == 0 &&
                   rot % (neighbours ? 4 : 8) == 0 && dim % 4 == 0 && q_rank % 4 == 0 && gate_width % 4 == 0 && a16(proj) &&
                   a16(q_out) && a16(wide) && a16(cache) && a16(gate);
  const int per_block = kThreads * (vec ? 4 : 1);
  a.query_blocks = heads > 0 ? (heads * (dim + rot) + per_block - 1) / per_block : 0;
  const int blocks = a.row_blocks + a.norm_blocks + a.query_blocks + (gate_width + per_block - 1) / per_block;
  PYRE_REQUIRE(blocks <= 65535, "latent_rows: too many columns");
  if (blocks == 0) return 0;
  PYRE_DISPATCH(proj_dt, TP, PYRE_DISPATCH(dt, T, {
    if (vec) hipLaunchKernelGGL((latent_rows_kernel<TP, T, 4>), dim3(n, blocks), dim3(kThreads), 0, stream, a);
    else hipLaunchKernelGGL((latent_rows_kernel<TP, T, 1>), dim3(n, blocks), dim3(kThreads), 0, stream, a);
  }));
  return check_launch("latent_rows");
}

extern "C" int pyre_head_matmul(const void* x, long x_token, long x_head, const void* w, void* out, long out_token,
                                long out_head, const float* gate, int dt, int n, int heads, int din, int dout,
                                hipStream_t stream) {
  PYRE_REQUIRE(known_dtype(dt) && x && w && out, "head_matmul: bad arguments");
  PYRE_REQUIRE(heads > 0 && heads <= 65535 && din > 0 && dout > 0 && x_token >= 0 && x_head >= din && out_head >= dout,
               "head_matmul: bad geometry");
  PYRE_REQUIRE((dout + 31) / 32 <= 65535, "head_matmul: heads of %d outputs are too wide", dout);
  if (n <= 0) return 0;
  const HeadProduct a{x, w, out, gate, x_token, x_head, out_token, out_head, n, heads, din, dout};
  const int E = dt == kBF16 ? 8 : 4;
  if (din % E == 0 && x_token % E == 0 && x_head % E == 0 && reinterpret_cast<uintptr_t>(x) % 16 == 0 && reinterpret_cast<uintptr_t>(w) % 16 == 0) {
    // (the float32 form has one order of sums whatever the number of tokens)
    if (n <= 64 || dt == kF32)
      PYRE_DISPATCH(dt, T, hipLaunchKernelGGL(head_matmul_few_kernel<T>, dim3((n + 31) / 32, heads, (dout + 31) / 32), dim3(kThreads), 0, stream, a));
    else
      hipLaunchKernelGGL(head_matmul_many_kernel, dim3((n + kTile - 1) / kTile, heads, (dout + kTile - 1) / kTile), dim3(kThreads), 0,
                         stream, a, dout % 8 == 0 && out_token % 8 == 0 && out_head % 8 == 0 && reinterpret_cast<uintptr_t>(out) % 16 == 0 &&
                             reinterpret_cast<uintptr_t>(gate) % 16 == 0);
    return check_launch("head_matmul");
  }
  PYRE_DISPATCH(dt, T, hipLaunchKernelGGL(head_matmul_any_kernel<T>, dim3(n, heads, (dout + kThreads - 1) / kThreads), dim3(kThreads), 0, stream, a));
  return check_launch("head_matmul");
}
