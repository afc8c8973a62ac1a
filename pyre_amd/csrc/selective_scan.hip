// A selective scan: per request and channel c a float32 state S [inner][N] that every token decays and adds to by numbers
// it makes itself, and reads:
//
//   u, g = the input product's columns (inner each);   x_t = silu(sum_j taps[j] u_(t - (T - 1) + j) + conv_b)
//   low, B, C = the columns of a second product, over x (rank, N, N)
//   dt = softplus(W_dt low + dt_b)                                              (one per channel)
//   S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;   y_c = sum_n S[c, n] C_n + D_c x_c;   out = y silu(g) out_scale
//
// ssm_conv   the convolution with its bias and silu, into rows of the engine's element type; the last T - 1 rows u of a
//            request are its state. A thread four channels (or one), every tap's input asked for before the first is used.
// ssm_low    the columns `low` as operands of the product that makes the step sizes: float32 as they are, or in 16-bit mode
//            as two bfloat16 numbers side by side, the rounded one and what the rounding left: against [W_dt | W_dt]
//            the product is then that of the unrounded numbers to 2^-17, since step sizes are 32-bit numbers.
// ssm_scan   the recurrence over each request's tokens of the step in their order. A block: one request, 32 or 16 channels,
//            eight or sixteen neighbouring lanes to a channel, lane l keeping the state's elements l NS .. l NS + NS - 1 in
//            registers. The tokens' numbers come 32 tokens at a time through LDS, brought and finished by waves of their
//            own; a tile's step sizes are made once (not by every lane) on the way there. The chain from token to token is
//            one multiply-add: the exponentials do not depend on it, and eight tokens are one piece of code without a
//            branch, so that they overlap. A token's sum over the state is joined by exchanges inside the vector unit.
// ssm_step   the same for steps of one token a request, with the step size's product inside: the eight lanes of a channel
//            share its row of W_dt, the second product's columns lie in LDS.
//
// A token's numbers are added in an order that its own sizes fix, and the state is walked token by token whatever the step
// holds, so a result does not depend on where a step begins. All arithmetic float32; exponentials of dt A as powers of two.
#include <type_traits>

#include "pyre_api.h"
#include "pyre_common.h"
#include "pyre_conv.h"

using namespace pyre;

namespace {

constexpr int kThreads = kConvThreads;
constexpr int kMaxTaps = 16;
constexpr int kLanes = 8;                    // lanes to a channel
constexpr int kChannels = kThreads / kLanes; // channels of a block
constexpr int kTile = 32;                    // tokens of a tile
constexpr int kMaxState = 256;
constexpr int kMaxSelected = 12288;          // floats of LDS for the second product's columns of a token

__device__ inline float silu_of(float z) { return z * __builtin_amdgcn_rcpf(1.f + expf(-z)); }

// log(1 + e^z) = max(z, 0) + log(1 + u), u = e^-|z| in (0, 1]; log(1 + u) = 2 atanh(s) with s = u / (2 + u) <= 1/3, whose
// power series 2 s (1 + s^2 / 3 + s^4 / 5 + ..) is cut behind s^16 (the rest is below 2^-29 of it): accurate to a few units in
// the last place however small u is, and without a branch.
__device__ inline float softplus_of(float z) {
  const float u = expf(-fabsf(z)), s = u * __builtin_amdgcn_rcpf(2.f + u), q = s * s;
  float p = 1.f / 17.f;
  p = fmaf(p, q, 1.f / 15.f), p = fmaf(p, q, 1.f / 13.f), p = fmaf(p, q, 1.f / 11.f), p = fmaf(p, q, 1.f / 9.f);
  p = fmaf(p, q, 1.f / 7.f), p = fmaf(p, q, 1.f / 5.f), p = fmaf(p, q, 1.f / 3.f), p = fmaf(p, q, 1.f);
  return fmaf(2.f * s, p, fmaxf(z, 0.f));
}

// A product as its partial sums; `col` counts from the first column of the part that is meant.
struct Columns {
  const void* data;
  int dt, n_partials;
  size_t stride;
  int ld, col0;
  const float* bias = nullptr;  // over all of the product's columns, or null
};
// The partial sums are added in their order, six of them asked for together.
__device__ inline float column(const Columns& p, size_t row, int col) {
  constexpr int kTogether = 6;
  const size_t at = row * p.ld + p.col0 + col;
  float v = 0.f;
  if (p.dt == kF32) {
    const float* src = static_cast<const float*>(p.data) + at;
#pragma unroll 1
    for (int i = 0; i < p.n_partials; i += kTogether) {
      float part[kTogether];
#pragma unroll
      for (int u = 0; u < kTogether; ++u) part[u] = i + u < p.n_partials ? src[(i + u) * p.stride] : 0.f;
#pragma unroll
      for (int u = 0; u < kTogether; ++u)
        if (i + u < p.n_partials) v += part[u];
    }
  } else {
#pragma unroll 1
    for (int i = 0; i < p.n_partials; ++i) v += to_float(static_cast<const bf16*>(p.data)[i * p.stride + at]);
  }
  return p.bias ? v + p.bias[p.col0 + col] : v;
}

// ---------------------------------------------------------------------------------------------
template <typename TX>
__global__ __launch_bounds__(kThreads) void ssm_conv_kernel(ConvIn in, const float* __restrict__ conv_b,
                                                            const int* __restrict__ state_slots,
                                                            const int* __restrict__ seq_of_token,
                                                            const int* __restrict__ q_start, TX* __restrict__ x) {
  const int n = blockIdx.x, seq = seq_of_token[n], run = n - q_start[seq], st = state_slots[seq];
  for (int ch = blockIdx.y * kThreads + threadIdx.x; ch < in.channels; ch += gridDim.y * kThreads)
    x[static_cast<size_t>(n) * in.channels + ch] = from_float<TX>(silu_of(conv_value(in, n, run, st, ch) + conv_b[ch]));
}

template <typename TP, typename TX>
__global__ __launch_bounds__(kThreads) void ssm_conv_vec_kernel(ConvIn in, const float* __restrict__ conv_b,
                                                                const int* __restrict__ state_slots,
                                                                const int* __restrict__ seq_of_token,
                                                                const int* __restrict__ q_start, TX* __restrict__ x,
                                                                float* shift_state) {
  const int n = blockIdx.x, seq = seq_of_token[n], run = n - q_start[seq], st = state_slots[seq];
  const int ch = 4 * (blockIdx.y * kThreads + threadIdx.x);
  if (ch >= in.channels) return;
  const float4 b = *reinterpret_cast<const float4*>(conv_b + ch);
  const float4 y = add4(conv_value4(in, static_cast<const TP*>(in.proj), n, run, st, ch, shift_state), b);
  Vec4<TX>::store(x + static_cast<size_t>(n) * in.channels + ch, float4{silu_of(y.x), silu_of(y.y), silu_of(y.z), silu_of(y.w)});
}

// ---------------------------------------------------------------------------------------------
template <typename TO>
__global__ __launch_bounds__(kThreads) void ssm_low_kernel(Columns sel, TO* __restrict__ out, int rank, int padded, size_t total) {
  const size_t i = static_cast<size_t>(blockIdx.x) * kThreads + threadIdx.x;
  if (i >= total) return;
  const size_t n = i / padded;
  const int r = static_cast<int>(i % padded);
  const float v = r < rank ? column(sel, n, r) : 0.f;
  if constexpr (sizeof(TO) == 4) {
    out[i] = v;
  } else {
    const bf16 high = from_float<bf16>(v);
    out[n * 2 * padded + r] = high;
    out[n * 2 * padded + padded + r] = from_float<bf16>(v - to_float(high));
  }
}

// ---------------------------------------------------------------------------------------------
struct ScanArgs {
  Columns z;            // W_dt low
  const float* dt_b;
  const void* x;        // [n][inner]
  int x_dt;
  Columns sel;          // B, then C
  Columns gate;
  const float* A2;      // [inner][N]: A log2(e)
  const float* D;
  float* state;         // [slots][inner][N]
  void* out;
  int out_dt;
  size_t out_ld;
  float out_scale;
  int inner, n_state;
};

// The sum over a group of L neighbouring lanes, in every lane of it (eight or sixteen).
template <int L>
__device__ inline float group_sum(float v) {
  v = lanes_sum<8>(v);
  if constexpr (L == 16) v += lane_exchange<0x140>(v);  // row_mirror: the other eight of a row of sixteen
  return v;
}

__device__ inline void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// A block: four waves that walk and four that do everything else, a tile ahead of them and a tile behind (they share the
// compute unit's four schedulers in pairs). In the round of tile i the walking waves turn its numbers in LDS into its sums;
// the others finish tile i - 1 (its sums, D x, the gate), put tile i + 1 into LDS (its step sizes made on the way) and send
// for tile i + 2. The two meet at one barrier a round, which waits for LDS alone.
// PLAIN: the usual case of many tokens, every product one float32 array without a bias, x and out bfloat16: the loads of a
// tile are then nothing but loads (addresses held inside the arrays, what is not there replaced by zero when it is used),
// so that all of them are on their way together.
template <int L, int NS, bool PLAIN>
__global__ __launch_bounds__(2 * kThreads) void ssm_scan_kernel(ScanArgs a, const int* __restrict__ q_start,
                                                                const int* __restrict__ state_slots) {
  constexpr int kCh = kThreads / L;                      // channels of a block
  constexpr int kStep = kThreads / kCh;                  // tokens that the helping waves cover at once
  constexpr int kMine = kTile / kStep;                   // (token, channel) pairs of a helping thread: tokens t, t + kStep, ..
  constexpr int kPad = NS * L;                           // elements of the state, padded
  constexpr int kBc = kTile * 2 * kPad / kThreads;       // numbers of B and C that a helping thread brings per tile
  constexpr int kHalf = (NS + 1) / 2;
  constexpr int kUnroll = NS <= 4 ? 8 : NS <= 8 ? 4 : 2;
  static_assert(kTile % 8 == 0 && kTile % kStep == 0 && kTile * 2 * kPad % kThreads == 0, "a tile is dealt evenly");
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float2(*steps)[kTile][kCh] = reinterpret_cast<float2(*)[kTile][kCh]>(lds);            // [2]: dt, dt x
  float(*bc)[kTile][2 * kPad] = reinterpret_cast<float(*)[kTile][2 * kPad]>(lds + 2 * 2 * kTile * kCh);  // [2], [lane][B | C]
  float(*ys)[kTile][kCh + 1] = reinterpret_cast<float(*)[kTile][kCh + 1]>(lds + 2 * 2 * kTile * kCh + 2 * kTile * 2 * kPad);  // [2]
  const int s = blockIdx.y, c0 = blockIdx.x * kCh, tid = threadIdx.x % kThreads;
  const int t_begin = q_start[s], t_end = q_start[s + 1], N = a.n_state;
  if (t_begin >= t_end) return;
  const int n_tiles = (t_end - t_begin + kTile - 1) / kTile;

  if (threadIdx.x >= kThreads) {  // the helping waves: thread -> channel fc, tokens ft, ft + kStep, ..
    const int fc = tid % kCh, ft = tid / kCh, fch = c0 + fc, fch_in = min(fch, a.inner - 1);
    const bool fin = fch < a.inner;
    const float dt_b = fin ? a.dt_b[fch] : 0.f, skip = fin ? a.D[fch] : 0.f;
    float z[kMine], g[kMine], b[kBc];                     // of the tile that is on its way
    typename std::conditional<PLAIN, bf16, float>::type x[kMine];
    float x1[kMine], g1[kMine], x0[kMine], g0[kMine];     // of the tile in LDS next, of the tile that is walked
    auto ask = [&](int tile) {
      const int t0 = t_begin + tile * kTile;
#pragma unroll
      for (int k = 0; k < kMine; ++k) {
        const size_t t = min(t0 + ft + k * kStep, t_end - 1);
        if constexpr (PLAIN) {
          z[k] = static_cast<const float*>(a.z.data)[t * a.z.ld + a.z.col0 + fch_in];
          x[k] = static_cast<const bf16*>(a.x)[t * a.inner + fch_in];
          g[k] = static_cast<const float*>(a.gate.data)[t * a.gate.ld + a.gate.col0 + fch_in];
        } else {
          z[k] = column(a.z, t, fch_in);
          x[k] = load_as_float(a.x, a.x_dt, t * a.inner + fch_in);
          g[k] = column(a.gate, t, fch_in);
        }
      }
#pragma unroll
      for (int k = 0; k < kBc; ++k) {
        const int i = tid + k * kThreads, col = i % (2 * kPad), n = min(col % kPad, N - 1);  // B of all elements, then C
        const size_t t = min(t0 + i / (2 * kPad), t_end - 1);
        if constexpr (PLAIN) b[k] = static_cast<const float*>(a.sel.data)[t * a.sel.ld + a.sel.col0 + (col < kPad ? n : N + n)];
        else b[k] = column(a.sel, t, col < kPad ? n : N + n);
      }
    };
    auto put = [&](int tile) {  // the tile that was on its way goes to LDS
      const int buf = tile & 1, left = t_end - t_begin - tile * kTile;
#pragma unroll
      for (int k = 0; k < kMine; ++k) {
        const int t = ft + k * kStep;
        x1[k] = to_float(x[k]), g1[k] = g[k];
        const float dt = t < left ? softplus_of(z[k] + dt_b) : 0.f;  // behind the last token: S times one, plus zero
        steps[buf][t][fc] = float2{dt, dt * x1[k]};
      }
#pragma unroll
      for (int k = 0; k < kBc; ++k) {
        const int i = tid + k * kThreads, t = i / (2 * kPad), col = i % (2 * kPad), n = col % kPad;
        bc[buf][t][(n / NS) * 2 * NS + n % NS + (col < kPad ? 0 : NS)] = n < N ? b[k] : 0.f;
      }
    };
    auto finish = [&](int tile, const float (&xs)[kMine], const float (&gs)[kMine]) {
      const int t0 = t_begin + tile * kTile;
#pragma unroll
      for (int k = 0; k < kMine; ++k) {
        const int t = ft + k * kStep;
        const float y = fmaf(skip, xs[k], ys[tile & 1][t][fc]) * silu_of(gs[k]) * a.out_scale;
        const size_t at = static_cast<size_t>(t0 + t) * a.out_ld + fch;
        if (fin && t0 + t < t_end) {
          if constexpr (PLAIN) static_cast<bf16*>(a.out)[at] = from_float<bf16>(y);
          else store_from_float(a.out, a.out_dt, at, y);
        }
      }
    };
    ask(0);
    put(0);
    if (n_tiles > 1) ask(1);
    lds_barrier();
    for (int i = 0; i < n_tiles; ++i) {
      if (i > 0) finish(i - 1, x0, g0);
#pragma unroll
      for (int k = 0; k < kMine; ++k) x0[k] = x1[k], g0[k] = g1[k];
      if (i + 1 < n_tiles) put(i + 1);
      if (i + 2 < n_tiles) ask(i + 2);
      lds_barrier();
    }
    finish(n_tiles - 1, x0, g0);
    return;
  }

  const int lane = tid & 63, part = lane % L, mine = (tid >> 6) * (kWave / L) + lane / L, ch = c0 + mine;
  float* st = a.state + (static_cast<size_t>(state_slots[s]) * a.inner + ch) * N;
  float S[NS], A2[NS];
#pragma unroll
  for (int j = 0; j < NS; ++j) {
    const int n = part * NS + j;
    const bool there = ch < a.inner && n < N;
    S[j] = there ? st[n] : 0.f;
    A2[j] = there ? a.A2[static_cast<size_t>(ch) * N + n] : 0.f;
  }
  lds_barrier();
  for (int i = 0; i < n_tiles; ++i) {
    const int buf = i & 1, nt = min(kTile, t_end - t_begin - i * kTile);
    for (int t8 = 0; t8 < nt; t8 += 8) {
      float keep = 0.f;  // lane part of a channel keeps the sum of token t8 + part: no branch between the tokens
#pragma unroll kUnroll
      for (int u = 0; u < 8; ++u) {
        const float2 step = steps[buf][t8 + u][mine];
        const float* row = &bc[buf][t8 + u][part * 2 * NS];
        float y0 = 0.f, y1 = 0.f;  // two halves of the lane's elements: with twice the lanes each is a lane's own
#pragma unroll
        for (int j = 0; j < NS; ++j) {
          S[j] = fmaf(__builtin_amdgcn_exp2f(step.x * A2[j]), S[j], step.y * row[j]);
          if (j < kHalf || L == 16) y0 = fmaf(S[j], row[NS + j], y0);
          else y1 = fmaf(S[j], row[NS + j], y1);
        }
        const float y = group_sum<L>(L == 16 || NS == 1 ? y0 : y0 + y1);
        keep = (part & 7) == u ? y : keep;
      }
      if (L == 8 || part < 8) ys[buf][t8 + (part & 7)][mine] = keep;
    }
    lds_barrier();
  }
#pragma unroll
  for (int j = 0; j < NS; ++j) {
    const int n = part * NS + j;
    if (ch < a.inner && n < N) st[n] = S[j];
  }
}
template <int L, int NS, bool PLAIN>
int launch_scan(const ScanArgs& a, const int* q_start, const int* state_slots, int n_seqs, hipStream_t stream) {
  constexpr int kCh = kThreads / L;
  constexpr size_t lds = sizeof(float) * 2 * kTile * (2 * kCh + 2 * NS * L + kCh + 1);
  static_assert(lds <= 160 * 1024, "a compute unit has 160 KB of LDS");
  static bool raised = lds <= 64 * 1024;
  if (!raised) {
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(&ssm_scan_kernel<L, NS, PLAIN>),
                            hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds)) != hipSuccess)
      return fail("ssm_scan: the device refuses %zu bytes of LDS", lds);
    raised = true;
  }
  hipLaunchKernelGGL((ssm_scan_kernel<L, NS, PLAIN>), dim3((a.inner + kCh - 1) / kCh, n_seqs), dim3(2 * kThreads), lds, stream, a,
                     q_start, state_slots);
  return 0;
}

// ---------------------------------------------------------------------------------------------
template <typename TW, int NS>
__global__ __launch_bounds__(kThreads) void ssm_step_kernel(ScanArgs a, const TW* __restrict__ dt_w, size_t dt_ld, int rank,
                                                            int vec, const int* __restrict__ state_slots) {
  extern __shared__ __attribute__((aligned(16))) float sel_s[];  // low, B, C of the token
  const int s = blockIdx.y, tid = threadIdx.x, part = tid % kLanes, ch = blockIdx.x * kChannels + tid / kLanes;
  const int N = a.n_state;
  const bool there = ch < a.inner;
  float* st = a.state + (static_cast<size_t>(state_slots[s]) * a.inner + ch) * N;
  float S[NS], A2[NS], x = 0.f, g = 0.f;
#pragma unroll
  for (int j = 0; j < NS; ++j) {  // asked for before the columns are waited for
    const int n = part * NS + j;
    S[j] = there && n < N ? st[n] : 0.f;
    A2[j] = there && n < N ? a.A2[static_cast<size_t>(ch) * N + n] : 0.f;
  }
  if (there) {
    x = load_as_float(a.x, a.x_dt, static_cast<size_t>(s) * a.inner + ch);
    g = column(a.gate, s, ch);
  }
  for (int i = tid; i < rank + 2 * N; i += kThreads) sel_s[i] = column(a.sel, s, i);
  __syncthreads();
  float z = 0.f;
  if (there) {
    const TW* row = dt_w + static_cast<size_t>(ch) * dt_ld;
    if (vec) {  // rank a multiple of four, rows on 16 bytes
      for (int r = 4 * part; r < rank; r += 4 * kLanes) {
        const float4 w = Vec4<TW>::load(row + r), l = *reinterpret_cast<const float4*>(sel_s + r);
        z = fmaf(w.x, l.x, z), z = fmaf(w.y, l.y, z), z = fmaf(w.z, l.z, z), z = fmaf(w.w, l.w, z);
      }
    } else {
      for (int r = part; r < rank; r += kLanes) z = fmaf(to_float(row[r]), sel_s[r], z);
    }
  }
  z = lanes_sum<kLanes>(z);
  const float dt = there ? softplus_of(z + a.dt_b[ch]) : 0.f, dtx = dt * x;
  const float* bs = sel_s + rank;
  float y = 0.f;
#pragma unroll
  for (int j = 0; j < NS; ++j) {
    const int n = part * NS + j;
    if (n < N) {
      S[j] = fmaf(__builtin_amdgcn_exp2f(dt * A2[j]), S[j], dtx * bs[n]);
      y = fmaf(S[j], bs[N + n], y);
      if (there) st[n] = S[j];
    }
  }
  y = lanes_sum<kLanes>(y);
  if (there && part == 0)
    store_from_float(a.out, a.out_dt, static_cast<size_t>(s) * a.out_ld + ch, fmaf(a.D[ch], x, y) * silu_of(g) * a.out_scale);
}

bool on16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

int check_scan(const char* what, const ScanArgs& a, int n_seqs) {
  PYRE_REQUIRE(known_dtype(a.x_dt) && known_dtype(a.out_dt) && known_dtype(a.sel.dt) && known_dtype(a.gate.dt), "%s: bad dtypes", what);
  PYRE_REQUIRE(a.sel.n_partials >= 1 && a.gate.n_partials >= 1 && a.inner > 0 && a.n_state > 0 && a.n_state <= kMaxState,
               "%s: %d channels with a state of %d (of at most %d) are not taken", what, a.inner, a.n_state, kMaxState);
  PYRE_REQUIRE(a.x && a.dt_b && a.A2 && a.D && a.state && a.out && n_seqs <= 65535, "%s: operands are missing, or %d requests are too many", what, n_seqs);
  return 0;
}

}  // namespace

extern "C" int pyre_ssm_conv(const void* proj, int proj_dt, int n_partials, long partial_stride, int ld, int col0,
                             const float* proj_bias, const float* taps_w, int taps, const float* conv_b, float* conv_state, const int* state_slots,
                             const int* seq_of_token, const int* q_start, int n_seqs, int single, void* x, int x_dt, int n,
                             int inner, hipStream_t stream) {
  PYRE_REQUIRE(known_dtype(proj_dt) && known_dtype(x_dt) && n_partials >= 1, "ssm_conv: bad dtypes");
  PYRE_REQUIRE(inner > 0 && taps_w && conv_b && taps >= 1 && taps <= kMaxTaps && (taps == 1 || conv_state),
               "ssm_conv: %d taps (of at most %d) need their weights, the bias and, beyond one, the state", taps, kMaxTaps);
  PYRE_REQUIRE(state_slots && seq_of_token && q_start && n_seqs >= 0 && n_seqs <= 65535, "ssm_conv: the step's arrays are needed");
  if (n <= 0) return 0;
  const ConvIn in{proj, proj_dt, n_partials, static_cast<size_t>(partial_stride), ld, col0, taps_w, taps, conv_state, inner,
                  proj_bias};
  if (taps <= kConvVecTaps && inner % 4 == 0 && ld % 4 == 0 && col0 % 4 == 0 && partial_stride % 4 == 0 && on16(proj) &&
      on16(x) && on16(taps_w) && on16(conv_b) && on16(conv_state) && on16(proj_bias)) {
    const dim3 grid(n, (inner / 4 + kThreads - 1) / kThreads);
    PYRE_DISPATCH(proj_dt, TP, PYRE_DISPATCH(x_dt, TX,
        hipLaunchKernelGGL((ssm_conv_vec_kernel<TP, TX>), grid, dim3(kThreads), 0, stream, in, conv_b, state_slots,
                           seq_of_token, q_start, static_cast<TX*>(x), single && taps > 1 ? conv_state : nullptr)));
    if (single) return check_launch("ssm_conv");
  } else {
    const int cols = (inner + kThreads - 1) / kThreads;
    PYRE_DISPATCH(x_dt, TX,
        hipLaunchKernelGGL(ssm_conv_kernel<TX>, dim3(n, cols < 64 ? cols : 64), dim3(kThreads), 0, stream, in, conv_b,
                           state_slots, seq_of_token, q_start, static_cast<TX*>(x)));
  }
  if (check_launch("ssm_conv")) return 1;
  if (taps > 1 && n_seqs > 0) {
    const int cols = (inner + kThreads - 1) / kThreads;
    hipLaunchKernelGGL(conv_state_update_kernel, dim3(n_seqs, cols < 64 ? cols : 64), dim3(kThreads), 0, stream, in,
                       conv_state, state_slots, q_start);
    return check_launch("conv_state_update");
  }
  return 0;
}

extern "C" int pyre_ssm_low(const void* sel, int sel_dt, int n_partials, long partial_stride, int ld, void* out, int out_dt,
                            int rank, int padded, int n, hipStream_t stream) {
  PYRE_REQUIRE(known_dtype(sel_dt) && known_dtype(out_dt) && n_partials >= 1, "ssm_low: bad dtypes");
  PYRE_REQUIRE(rank > 0 && padded >= rank && ld >= rank, "ssm_low: %d columns do not fit rows of %d", rank, padded);
  if (n <= 0) return 0;
  const Columns cols{sel, sel_dt, n_partials, static_cast<size_t>(partial_stride), ld, 0};
  const size_t total = static_cast<size_t>(n) * padded;
  PYRE_DISPATCH(out_dt, TO,
      hipLaunchKernelGGL(ssm_low_kernel<TO>, dim3((total + kThreads - 1) / kThreads), dim3(kThreads), 0, stream, cols,
                         static_cast<TO*>(out), rank, padded, total));
  return check_launch("ssm_low");
}

// Elements of the state to a lane: the smallest form that holds them.
#define PYRE_SSM_FORMS(N, LAUNCH)                 \
  do {                                            \
    const int per_lane = ((N) + kLanes - 1) / kLanes; \
    if (per_lane <= 1) LAUNCH(1);                 \
    else if (per_lane <= 2) LAUNCH(2);            \
    else if (per_lane <= 3) LAUNCH(3);            \
    else if (per_lane <= 4) LAUNCH(4);            \
    else if (per_lane <= 6) LAUNCH(6);            \
    else if (per_lane <= 8) LAUNCH(8);            \
    else if (per_lane <= 16) LAUNCH(16);          \
    else LAUNCH(32);                              \
  } while (0)

extern "C" int pyre_ssm_scan(const void* z, int z_dt, int z_partials, long z_stride, const float* dt_b, const void* x, int x_dt,
                             const void* sel, int sel_dt, int sel_partials, long sel_stride, int sel_ld, int b0,
                             const void* proj, int proj_dt, int proj_partials, long proj_stride, int proj_ld, const float* proj_bias,
                             int g0,
                             const float* A2, const float* D, float* state, const int* q_start, const int* state_slots,
                             int n_seqs, float out_scale, void* out, int out_dt, long out_ld, int inner, int n_state,
                             hipStream_t stream) {
  const ScanArgs a{{z, z_dt, z_partials, static_cast<size_t>(z_stride), inner, 0}, dt_b, x, x_dt,
                   {sel, sel_dt, sel_partials, static_cast<size_t>(sel_stride), sel_ld, b0},
                   {proj, proj_dt, proj_partials, static_cast<size_t>(proj_stride), proj_ld, g0, proj_bias},
                   A2, D, state, out, out_dt, static_cast<size_t>(out_ld), out_scale, inner, n_state};
  if (int rc = check_scan("ssm_scan", a, n_seqs)) return rc;
  PYRE_REQUIRE(z && known_dtype(z_dt) && z_partials >= 1 && q_start && state_slots, "ssm_scan: the step sizes' product and the step's arrays are needed");
  if (n_seqs <= 0) return 0;
  // eight lanes to a channel, or sixteen where blocks of the former would leave half of the compute units idle (a token
  // of a wave is then shorter; the same sums in the same order)
  const int blocks8 = (inner + kThreads / 8 - 1) / (kThreads / 8);
  const bool wide = static_cast<long>(blocks8) * n_seqs <= compute_units() / 2;
  const bool plain = z_dt == kF32 && sel_dt == kF32 && proj_dt == kF32 && z_partials == 1 && sel_partials == 1 &&
                     proj_partials == 1 && !proj_bias && x_dt == kBF16 && out_dt == kBF16;
#define PYRE_SCAN(L, NS)                                                                                            \
  do {                                                                                                              \
    if (int rc = plain ? launch_scan<L, NS, true>(a, q_start, state_slots, n_seqs, stream)                          \
                       : launch_scan<L, NS, false>(a, q_start, state_slots, n_seqs, stream))                        \
      return rc;                                                                                                    \
  } while (0)
#define PYRE_SCAN8(NS) PYRE_SCAN(8, NS)
  if (wide && n_state > 8 && n_state <= 16) PYRE_SCAN(16, 1);
  else if (wide && n_state > 24 && n_state <= 32) PYRE_SCAN(16, 2);
  else if (wide && n_state > 48 && n_state <= 64) PYRE_SCAN(16, 4);
  else if (wide && n_state > 64 && n_state <= 128) PYRE_SCAN(16, 8);
  else if (wide && n_state > 128) PYRE_SCAN(16, 16);
  else PYRE_SSM_FORMS(n_state, PYRE_SCAN8);
#undef PYRE_SCAN8
#undef PYRE_SCAN
  return check_launch("ssm_scan");
}

extern "C" int pyre_ssm_step(const void* dt_w, int dt_w_dt, long dt_ld, const float* dt_b, const void* x, int x_dt,
                             const void* sel, int sel_dt, int sel_partials, long sel_stride, int sel_ld, int rank,
                             const void* proj, int proj_dt, int proj_partials, long proj_stride, int proj_ld, const float* proj_bias,
                             int g0,
                             const float* A2, const float* D, float* state, const int* state_slots, int n_seqs,
                             float out_scale, void* out, int out_dt, long out_ld, int inner, int n_state, hipStream_t stream) {
  const ScanArgs a{{nullptr, kF32, 1, 0, inner, 0}, dt_b, x, x_dt,
                   {sel, sel_dt, sel_partials, static_cast<size_t>(sel_stride), sel_ld, 0},
                   {proj, proj_dt, proj_partials, static_cast<size_t>(proj_stride), proj_ld, g0, proj_bias},
                   A2, D, state, out, out_dt, static_cast<size_t>(out_ld), out_scale, inner, n_state};
  if (int rc = check_scan("ssm_step", a, n_seqs)) return rc;
  PYRE_REQUIRE(dt_w && known_dtype(dt_w_dt) && rank > 0 && dt_ld >= rank && rank + 2 * n_state <= kMaxSelected && state_slots,
               "ssm_step: a rank of %d beside a state of %d is not taken", rank, n_state);
  if (n_seqs <= 0) return 0;
  const dim3 grid((inner + kChannels - 1) / kChannels, n_seqs);
  const size_t lds = sizeof(float) * (rank + 2 * n_state);
  const int vec = rank % 4 == 0 && dt_ld % 4 == 0 && on16(dt_w);
#define PYRE_STEP(NS) \
  hipLaunchKernelGGL((ssm_step_kernel<TW, NS>), grid, dim3(kThreads), lds, stream, a, static_cast<const TW*>(dt_w), \
                     static_cast<size_t>(dt_ld), rank, vec, state_slots)
  PYRE_DISPATCH(dt_w_dt, TW, PYRE_SSM_FORMS(n_state, PYRE_STEP));
#undef PYRE_STEP
  return check_launch("ssm_step");
}
