// Linear memories: a matrix S [n, v] a head that is carried from token to token,
//     S_t = S' + k w^T,  S' = e^g S_(t-1),  o = S_t^T q,    w = write * val,  or with DELTA  w = write * (val - S'^T k),
// g a number a head or, with KEYED, one for every row of S (a key channel), and what stands before and after them in a mixer:
//   memory_inputs   a short causal convolution over time with silu, unit vectors a head, decays and write weights
//   channel_decays  the decays of every key channel through a bottleneck
//   turn_heads      queries and keys turned by the position, in place
//   memory_walk     the recurrence token by token (decoded tokens, short runs)
//   memory_pairs (memory_pairs_keyed), memory_scan   the same for long runs, 64 tokens at a time on the matrix unit
//   gated_norm      skip, gate and norm, up to what the output product reads
// Everything is float32. State lies by position: the token at position p reads place (p - 1) & 1 of S's two (nothing at
// p = 0) and writes place p & 1; the convolution's input at position p lies at place p mod taps. A step of single tokens
// that is run twice reads the same both times.
#include "common.h"

TNX_DEFINE_ERROR_API

namespace {

__device__ __forceinline__ float silu(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// ------------------------------------------------------------------------------------------ what a memory reads

struct InputArgs {
  const float* proj;        // [T, ld]
  int ld, conv_at, channels;
  const float* w;           // [taps, channels]
  const float* bias;        // [channels] or null
  float* state;             // [slots, taps, channels]
  int taps;
  const int* positions;
  const int* token_request;
  const int* run_start;
  const int* slots;
  int unit_size, unit_count, scaled;      // the first unit_count channels are heads of unit_size, made unit vectors
  float scale;                            // on the first `scaled` channels
  float* u;                 // [T, u_ld]
  int u_ld;
  int heads, dt_at, write_at;             // write_at < 0: the write weight is dt
  const float* rate;        // [H]
  const float* dt_bias;     // [H]
  float* log_decay;         // [T, H]
  float* write;             // [T, H]
  int tokens, write_state;  // write_state: every run of the step is one token, so the state is written here
};

// A wave takes a piece of the channels for `per` consecutive tokens of the step: LANES: 256 channels, four a lane, where
// unit heads are 4 * LANES elements (the sum of squares is then one over LANES lanes); LANES = 0, any sizes: a unit head,
// or 256 channels, element lane + 64 e a lane. The inputs of the last taps - 1 tokens stay in registers while the run
// goes on. Behind the channels' pieces come those of the gates, 64 heads a wave. TAPS 0: any number, read again for
// every token.
template <int LANES, int TAPS>
__global__ void __launch_bounds__(256) memory_inputs_kernel(InputArgs a, int pieces, int per) {
  const int lane = threadIdx.x & 63;
  const int piece = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int t0 = blockIdx.y * per, t1 = min(a.tokens, t0 + per);
  if (piece >= pieces) {      // the gates
    const int head = 64 * (piece - pieces) + lane;
    if (head >= a.heads) return;
    for (int t = t0; t < t1; ++t) {
      const float* row = a.proj + (size_t)t * a.ld;
      const float dt = softplus(row[a.dt_at + head] + a.dt_bias[head]);
      a.log_decay[(size_t)t * a.heads + head] = a.rate[head] * dt;
      a.write[(size_t)t * a.heads + head] = a.write_at >= 0 ? 1.f / (1.f + expf(-row[a.write_at + head])) : dt;
    }
    return;
  }
  // this lane's channels: at[e], in[e]
  int at[4];
  bool in[4];
  bool unit = false;
  if (LANES > 0) {
    const int c = 256 * piece + 4 * lane;
#pragma unroll
    for (int e = 0; e < 4; ++e) at[e] = c + e, in[e] = c + e < a.channels;
    unit = c < a.unit_count;
  } else {
    const int unit_pieces = a.unit_size > 0 ? a.unit_count / a.unit_size : 0;
    unit = piece < unit_pieces;
    const int first = unit ? piece * a.unit_size : a.unit_count + 256 * (piece - unit_pieces);
    const int end = unit ? first + a.unit_size : a.channels;
#pragma unroll
    for (int e = 0; e < 4; ++e) at[e] = first + lane + 64 * e, in[e] = at[e] < end;
  }
  const bool whole = LANES > 0 && in[3] && ((a.channels | a.u_ld) & 3) == 0;       // four neighbours, 16 bytes aligned
  constexpr int BACK = TAPS > 1 ? TAPS - 1 : 1;
  float taps_w[TAPS > 0 ? TAPS : 1][4], bias[4], scale[4], before[BACK][4];
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const int c = in[e] ? at[e] : 0;
    bias[e] = a.bias && in[e] ? a.bias[c] : 0.f;
    scale[e] = at[e] < a.scaled ? a.scale : 1.f;
#pragma unroll
    for (int j = 0; j < (TAPS > 0 ? TAPS : 0); ++j) taps_w[j][e] = in[e] ? a.w[(size_t)j * a.channels + c] : 0.f;
#pragma unroll
    for (int b = 0; b < BACK; ++b) before[b][e] = 0.f;
  }
  const float* x = a.proj + a.conv_at;
  const bool vec = whole && ((a.ld | a.conv_at) & 3) == 0;
  auto load_row = [&](int t, float (&v)[4]) {
    const float* row = x + (size_t)t * a.ld;
    if (vec) {
      const f32x4 got = *(const f32x4*)(row + at[0]);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = got[e];
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = in[e] ? row[at[e]] : 0.f;
    }
  };
  auto load_back = [&](int t, int i, int p, int back, const float* mine, float (&v)[4]) {      // the input `back` tokens ago
    if (back <= i) {
      load_row(t - back, v);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = back <= p && in[e] ? mine[(size_t)((p - back) % a.taps) * a.channels + at[e]] : 0.f;
    }
  };
  float next[4];
  if (t0 < t1) load_row(t0, next);
  for (int t = t0; t < t1; ++t) {
    float now[4], acc[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) now[e] = next[e], acc[e] = bias[e];
    if (t + 1 < t1) load_row(t + 1, next);
    const int r = a.token_request[t], i = t - a.run_start[r], p = a.positions[t];
    float* mine = a.state ? a.state + (size_t)a.slots[r] * a.taps * a.channels : nullptr;
    if (TAPS > 0) {
      if (TAPS > 1 && (t == t0 || i == 0)) {
#pragma unroll
        for (int b = 1; b < TAPS; ++b) load_back(t, i, p, b, mine, before[b - 1]);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
#pragma unroll
        for (int b = TAPS - 1; b >= 1; --b) acc[e] = fmaf(taps_w[TAPS - 1 - b][e], before[b - 1][e], acc[e]);
        acc[e] = fmaf(taps_w[TAPS > 0 ? TAPS - 1 : 0][e], now[e], acc[e]);
#pragma unroll
        for (int b = BACK - 1; b >= 1; --b) before[b][e] = before[b - 1][e];
        before[0][e] = now[e];
      }
    } else {
      for (int b = a.taps - 1; b >= 0; --b) {
        float v[4];
        load_back(t, i, p, b, mine, v);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          acc[e] = fmaf(in[e] ? a.w[(size_t)(a.taps - 1 - b) * a.channels + at[e]] : 0.f, v[e], acc[e]);
      }
    }
    if (a.write_state && a.taps > 1) {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (in[e]) mine[(size_t)(p % a.taps) * a.channels + at[e]] = now[e];
    }
    float sum = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      acc[e] = in[e] ? silu(acc[e]) : 0.f;
      sum += acc[e] * acc[e];
    }
    if (LANES == 0) {
      if (unit) sum = wave_sum(sum);
    } else if (a.unit_count > 0) {
      sum += lane_dpp<TNX_DPP_XOR1>(sum);
      sum += lane_dpp<TNX_DPP_XOR2>(sum);
      sum += lane_dpp<TNX_DPP_HALF_MIRROR>(sum);
      sum += lane_dpp<TNX_DPP_MIRROR>(sum);
      if (LANES >= 32) {
        unsigned lo, hi;
        swap_rows(__float_as_uint(sum), lo, hi);
        sum = __uint_as_float(lo) + __uint_as_float(hi);
      }
      if (LANES >= 64) {
        unsigned lo, hi;
        swap_halves(__float_as_uint(sum), lo, hi);
        sum = __uint_as_float(lo) + __uint_as_float(hi);
      }
    }
    const float f = unit ? 1.f / sqrtf(sum + 1e-6f) : 1.f;
    float* out = a.u + (size_t)t * a.u_ld;
    if (whole) {
      f32x4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = acc[e] * f * scale[e];
      *(f32x4*)(out + at[0]) = o;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (in[e]) out[at[e]] = acc[e] * f * scale[e];
    }
  }
}

// the last taps - 1 inputs of every run, after the launch that read the state
__global__ void __launch_bounds__(256) memory_state_kernel(InputArgs a) {
  const int r = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  const int first = a.run_start[r], n = a.run_start[r + 1] - first;
  if (c >= a.channels || n <= 0) return;
  float* mine = a.state + (size_t)a.slots[r] * a.taps * a.channels;
  for (int i = max(0, n - (a.taps - 1)); i < n; ++i)
    mine[(size_t)(a.positions[first + i] % a.taps) * a.channels + c] = a.proj[(size_t)(first + i) * a.ld + a.conv_at + c];
}

// ln(1 + x) for x in [0, 1] (Goldberg, "What Every Computer Scientist Should Know About Floating-Point Arithmetic", theorem
// 4: the rounding of 1 + x drops out of x ln(u) / (u - 1) with u = 1 + x as rounded)
__device__ __forceinline__ float log_one_plus(float x) {
  const float u = 1.f + x;
  return u == 1.f ? x : __fdividef(x * __logf(u), u - 1.f);
}
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log_one_plus(expf(-fabsf(z))); }

// log_sigmoid(low w^T + bias) / tau for every key channel. A block takes 256 channels, one a thread, and TT tokens, whose
// `low` goes through LDS 16 elements at a time.
struct DecayArgs {
  const float* low;         // [T, low_ld]
  long long low_ld;
  const void* w;            // [channels, rank]
  const float* bias;        // [channels]
  float over_tau;
  float* out;               // [T, channels]
  int tokens, channels, rank;
};

template <typename W, int TT>
__global__ void __launch_bounds__(256) channel_decays_kernel(DecayArgs a) {
  __shared__ __attribute__((aligned(16))) float low[TT * 16];
  const int c = blockIdx.x * 256 + threadIdx.x, t0 = blockIdx.y * TT;
  const bool in = c < a.channels;
  const W* row = (const W*)a.w + (size_t)(in ? c : 0) * a.rank;
  const float b = in ? a.bias[c] : 0.f;
  float acc[TT];
#pragma unroll
  for (int t = 0; t < TT; ++t) acc[t] = 0.f;
  for (int r0 = 0; r0 < a.rank; r0 += 16) {
    if (r0 > 0) __syncthreads();
    if (threadIdx.x < TT * 16) {
      const int t = threadIdx.x >> 4, e = threadIdx.x & 15;
      low[threadIdx.x] = t0 + t < a.tokens && r0 + e < a.rank ? a.low[(size_t)(t0 + t) * a.low_ld + r0 + e] : 0.f;
    }
    float w[16];
    if (a.rank % 16 == 0) {
      typedef W eight __attribute__((ext_vector_type(8)));
      const eight w0 = *(const eight*)(row + r0), w1 = *(const eight*)(row + r0 + 8);
#pragma unroll
      for (int e = 0; e < 8; ++e) w[e] = to_f32(w0[e]), w[8 + e] = to_f32(w1[e]);
    } else {
#pragma unroll
      for (int e = 0; e < 16; ++e) w[e] = in && r0 + e < a.rank ? to_f32(row[r0 + e]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < TT; ++t)
#pragma unroll
      for (int e = 0; e < 16; e += 4) {
        const f32x4 l = *(const f32x4*)(low + 16 * t + e);
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[t] = fmaf(w[e + i], l[i], acc[t]);
      }
  }
  if (!in) return;
#pragma unroll
  for (int t = 0; t < TT; ++t)
    if (t0 + t < a.tokens) a.out[(size_t)(t0 + t) * a.channels + c] = log_sigmoid(acc[t] + b) * a.over_tau;
}

// The first 2 half elements of `heads` heads of n, from column `at` of a row on, turned by the token's position, in place:
// a block a token, a thread a pair; the token's sines and cosines are made once.
__global__ void __launch_bounds__(256) turn_heads_kernel(float* __restrict__ x, int ld, int at, int heads, int n,
                                                         const float* __restrict__ freqs, int half, int interleaved,
                                                         const int* __restrict__ positions) {
  __shared__ float cosines[128], sines[128];
  const int t = blockIdx.x;
  const float pos = (float)positions[t];
  for (int i = threadIdx.x; i < half; i += 256) sincosf(pos * freqs[i], &sines[i], &cosines[i]);
  __syncthreads();
  float* row = x + (size_t)t * ld + at;
  for (int f = threadIdx.x; f < heads * half; f += 256) {
    const int head = f / half, i = f - head * half;
    float* u = row + head * n + (interleaved ? 2 * i : i);
    float* v = u + (interleaved ? 1 : half);
    const float a = *u, b = *v, c = cosines[i], s = sines[i];
    *u = a * c - b * s;
    *v = b * c + a * s;
  }
}

// ------------------------------------------------------------------------------------------ the memory, token by token

// how a memory's S' and w come about
constexpr int PLAIN = 0, DELTA_RULE = 1, KEYED = 2;

struct WalkArgs {
  const float* u;           // [T, ld]
  int ld, q_at, k_at, v_at;
  const float* log_decay;   // [T, H]; [H] with decay_ld = 0: the same for every token; KEYED: [T, H n]
  int decay_ld;             // elements from one token's decays to the next's
  const float* write;       // [T, H] or null: 1
  const int* run_start;     // [R + 1]
  const int* cached;        // [R]
  const int* slots;         // [R]
  float* memory;            // [slots, 2, H, v, n]
  float* out;               // [T, H v]
  int heads, groups, n, v;
  int longest;              // runs of more tokens than this are other kernels' (0: none are)
};

template <bool ALIGNED>
__device__ __forceinline__ f32x4 load4(const float* p, int valid) {      // the first `valid` of four elements, zeros behind
  f32x4 r = {0.f, 0.f, 0.f, 0.f};
  if (valid <= 0) return r;
  if (ALIGNED) return *(const f32x4*)p;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (e < valid) r[e] = p[e];
  return r;
}

// sums over the 16 lanes of a row of lanes
__device__ __forceinline__ float sum16(float x) {
  x += lane_dpp<TNX_DPP_XOR1>(x);
  x += lane_dpp<TNX_DPP_XOR2>(x);
  x += lane_dpp<TNX_DPP_HALF_MIRROR>(x);
  x += lane_dpp<TNX_DPP_MIRROR>(x);
  return x;
}

// grid: requests * heads * column blocks; a block is four waves and 16 columns of S. In a wave the 16 lanes of a row of
// lanes share a column (column 16 b + 4 w + lane / 16): lane % 16 holds its rows NR (lane % 16) + j, j < NR. CH tokens a
// chunk go through LDS, the next chunk's loads under way meanwhile, a token's operands read a token ahead.
// With DELTA S^T k, S^T q and k . q are summed side by side from the S that came in, and S'^T q = S^T q + w (k . q).
// KEYED: a token's decays go through LDS as its keys do. Without DELTA S decays by S + S (e^g - 1): a factor just below one,
// rounded to float32, would be off by the same amount at every token, and a memory of hundreds of tokens with it.
template <int NR, int CH, int MODE, bool ALIGNED>
__global__ void __launch_bounds__(256) memory_walk_kernel(WalkArgs a, int column_blocks) {
  constexpr bool DELTA = MODE == DELTA_RULE;
  constexpr int np = 16 * NR;                             // a token's queries (and keys) in LDS, zeros behind n
  constexpr int PT = np / 4;                              // 16-byte pieces of a token's queries
  constexpr int QN = (CH * PT + 255) / 256;               // pieces of queries (and keys) a thread and chunk
  __shared__ __attribute__((aligned(16))) float qs[CH * np];
  __shared__ __attribute__((aligned(16))) float ks[CH * np];
  __shared__ __attribute__((aligned(16))) float ds[MODE == KEYED ? CH * np : 4];      // e^g - 1, row by row of S
  __shared__ __attribute__((aligned(16))) float vs[CH * 16];
  __shared__ float kp[CH], wr[CH];                        // e^g (DELTA) or e^g - 1, write
  const int cb = blockIdx.x % column_blocks, rh = blockIdx.x / column_blocks;
  const int r = rh / a.heads, head = rh - r * a.heads;
  const int group = head / (a.heads / a.groups);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int grp = lane & 15;
  const int start = a.run_start[r], count = a.run_start[r + 1] - start;
  const int have = a.cached[r], slot = a.slots[r];
  if (count <= 0 || (a.longest > 0 && count > a.longest)) return;
  const int col = 16 * cb + 4 * wave + (lane >> 4);
  const bool col_ok = col < a.v;
  float S[NR];
  const int from = (have - 1) & 1, to = (have + count - 1) & 1;
  const size_t head_at = (size_t)slot * 2 * a.heads + head;        // + place * heads
  const float* Sp = a.memory + ((head_at + (size_t)from * a.heads) * a.v + (col_ok ? col : 0)) * a.n;
  const bool live = have > 0 && col_ok;
  if (NR % 4 == 0) {
#pragma unroll
    for (int j = 0; j < NR; j += 4) {
      const int d = grp * NR + j;
      const f32x4 got = load4<ALIGNED>(Sp + d, live ? a.n - d : 0);
#pragma unroll
      for (int e = 0; e < 4; ++e) S[j + (NR % 4 == 0 ? e : 0)] = got[e];
    }
  } else {
#pragma unroll
    for (int j = 0; j < NR; ++j) S[j] = live && grp * NR + j < a.n ? Sp[grp * NR + j] : 0.f;
  }
  f32x4 rq[QN], rk[QN], rd[MODE == KEYED ? QN : 1], rv = {0.f, 0.f, 0.f, 0.f};
  float rkeep = 1.f, rwrite = 0.f;
  auto fetch = [&](int t0) {
    const int len = min(CH, count - t0);
#pragma unroll
    for (int u = 0; u < QN; ++u) {
      const int f = threadIdx.x + 256 * u, t = f / PT, d = 4 * (f - t * PT);
      const bool in = f < CH * PT && t < len;
      const float* row = a.u + (size_t)(start + t0 + (in ? t : 0)) * a.ld + group * a.n + d;
      rq[u] = load4<ALIGNED>(row + a.q_at, in ? a.n - d : 0);
      rk[u] = load4<ALIGNED>(row + a.k_at, in ? a.n - d : 0);
      if (MODE == KEYED)
        rd[MODE == KEYED ? u : 0] =
            load4<ALIGNED>(a.log_decay + (size_t)(start + t0 + (in ? t : 0)) * a.decay_ld + head * a.n + d, in ? a.n - d : 0);
    }
    if (threadIdx.x < CH * 4) {                            // a token's 16 values: four pieces
      const int t = threadIdx.x >> 2, c = 16 * cb + 4 * (threadIdx.x & 3);
      const bool in = t < len;
      rv = load4<ALIGNED>(a.u + (size_t)(start + t0 + (in ? t : 0)) * a.ld + a.v_at + head * a.v + c, in ? a.v - c : 0);
    }
    if (threadIdx.x < CH) {
      const bool in = threadIdx.x < len;
      const size_t t = start + t0 + (in ? threadIdx.x : 0);
      if (MODE != KEYED) rkeep = in ? (DELTA ? expf(a.log_decay[t * a.decay_ld + head]) : expm1f(a.log_decay[t * a.decay_ld + head])) : 0.f;
      rwrite = in ? (a.write ? a.write[t * a.heads + head] : 1.f) : 0.f;
    }
  };
  auto stash = [&]() {
#pragma unroll
    for (int u = 0; u < QN; ++u) {
      const int f = threadIdx.x + 256 * u;                // piece f of the chunk: token f / PT, elements 4 (f % PT) on
      if (f < CH * PT) {
        *(f32x4*)(qs + 4 * f) = rq[u];
        *(f32x4*)(ks + 4 * f) = rk[u];
        if (MODE == KEYED) {
          f32x4 e4;
#pragma unroll
          for (int e = 0; e < 4; ++e) e4[e] = expm1f(rd[MODE == KEYED ? u : 0][e]);
          *(f32x4*)(ds + 4 * f) = e4;
        }
      }
    }
    if (threadIdx.x < CH * 4) *(f32x4*)(vs + 4 * threadIdx.x) = rv;
    if (threadIdx.x < CH) kp[threadIdx.x] = rkeep, wr[threadIdx.x] = rwrite;
  };
  fetch(0);
  stash();
  __syncthreads();
  for (int t0 = 0; t0 < count; t0 += CH) {
    const int len = min(CH, count - t0);
    const bool more = t0 + CH < count;
    if (more) fetch(t0 + CH);                             // under way while this chunk is worked on
    float q_n[NR], k_n[NR], d_n[MODE == KEYED ? NR : 1], val_n, keep_n, write_n;
    auto read = [&](int t) {
      const float* q = qs + t * np + grp * NR;
      const float* k = ks + t * np + grp * NR;
#pragma unroll
      for (int j = 0; j < NR; ++j) {
        q_n[j] = q[j], k_n[j] = k[j];
        if (MODE == KEYED) d_n[MODE == KEYED ? j : 0] = ds[t * np + grp * NR + j];
      }
      val_n = vs[t * 16 + 4 * wave + (lane >> 4)];
      keep_n = kp[t];
      write_n = wr[t];
    };
    auto token = [&](int t, bool last) {
      float q[NR], k[NR], d[MODE == KEYED ? NR : 1];
#pragma unroll
      for (int j = 0; j < NR; ++j) {
        q[j] = q_n[j], k[j] = k_n[j];
        if (MODE == KEYED) d[MODE == KEYED ? j : 0] = d_n[MODE == KEYED ? j : 0];
      }
      const float val = val_n, keep = keep_n, write = write_n;
      if (!last) read(t + 1);
      float o = 0.f;
      if (DELTA) {
        float sk = 0.f, sq = 0.f, kq = 0.f;
#pragma unroll
        for (int j = 0; j < NR; ++j) {
          S[j] *= keep;
          sk += S[j] * k[j];
          sq += S[j] * q[j];
          kq += k[j] * q[j];
        }
        sk = sum16(sk), sq = sum16(sq), kq = sum16(kq);
        const float w = write * (val - sk);
#pragma unroll
        for (int j = 0; j < NR; ++j) S[j] += k[j] * w;
        o = sq + w * kq;
      } else {
        const float w = write * val;
#pragma unroll
        for (int j = 0; j < NR; ++j) {
          S[j] = fmaf(k[j], w, fmaf(MODE == KEYED ? d[MODE == KEYED ? j : 0] : keep, S[j], S[j]));
          o += S[j] * q[j];
        }
        o = sum16(o);
      }
      if (grp == 0 && col_ok) a.out[((size_t)(start + t0 + t) * a.heads + head) * a.v + col] = o;
    };
    read(0);
    if (len == CH) {        // a whole chunk: a count the compiler knows
#pragma unroll 4
      for (int t = 0; t < CH; ++t) token(t, t == CH - 1);
    } else {
      for (int t = 0; t < len; ++t) token(t, t == len - 1);
    }
    __syncthreads();        // before the next chunk takes the place of what this one read
    if (more) {
      stash();
      __syncthreads();
    }
  }
  if (!col_ok) return;
  float* Sw = a.memory + ((head_at + (size_t)to * a.heads) * a.v + col) * a.n;
  if (ALIGNED && NR % 4 == 0) {
#pragma unroll
    for (int j = 0; j < NR; j += 4) {
      f32x4 out;
#pragma unroll
      for (int e = 0; e < 4; ++e) out[e] = S[j + (NR % 4 == 0 ? e : 0)];
      if (grp * NR + j < a.n) *(f32x4*)(Sw + grp * NR + j) = out;
    }
    return;
  }
#pragma unroll
  for (int j = 0; j < NR; ++j)
    if (grp * NR + j < a.n) Sw[grp * NR + j] = S[j];
}

template <int NR, int MODE>
void launch_walk(const WalkArgs& a, int requests, bool singles, bool aligned, hipStream_t stream) {
  constexpr int CH = NR == 16 ? 16 : 32;
  const int column_blocks = (a.v + 15) / 16;
  const dim3 grid(requests * a.heads * column_blocks);
  if (singles) {
    if (aligned)
      memory_walk_kernel<NR, 1, MODE, true><<<grid, 256, 0, stream>>>(a, column_blocks);
    else
      memory_walk_kernel<NR, 1, MODE, false><<<grid, 256, 0, stream>>>(a, column_blocks);
  } else {
    if (aligned)
      memory_walk_kernel<NR, CH, MODE, true><<<grid, 256, 0, stream>>>(a, column_blocks);
    else
      memory_walk_kernel<NR, CH, MODE, false><<<grid, 256, 0, stream>>>(a, column_blocks);
  }
}

template <int MODE>
void launch_walk_sized(const WalkArgs& a, int requests, bool singles, bool aligned, hipStream_t stream) {
  const int rows16 = (a.n + 15) / 16;
  if (rows16 <= 2)
    launch_walk<2, MODE>(a, requests, singles, aligned, stream);
  else if (rows16 <= 4)
    launch_walk<4, MODE>(a, requests, singles, aligned, stream);
  else if (rows16 <= 8)
    launch_walk<8, MODE>(a, requests, singles, aligned, stream);
  else
    launch_walk<16, MODE>(a, requests, singles, aligned, stream);
}

// ------------------------------------------------------------------------------------------ the memory, chunk by chunk

// 64 tokens at a time, with c_i = g_1 + ... + g_i the sum of the chunk's log decays up to token i and S the state the
// chunk begins with. Token i's write w_i and result o_i follow from S and the tokens before it in the chunk:
//     DELTA:  w_i = write_i (val_i - e^c_i S^T k_i - sum_{j<i} e^(c_i - c_j) (k_i . k_j) w_j),   otherwise write_i val_i
//     o_i = e^c_i S^T q_i + sum_{j<=i} e^(c_i - c_j) (q_i . k_j) w_j
//     the state after the chunk: e^c_64 S + sum_j e^(c_64 - c_j) k_j w_j^T
// With DELTA the w are the solution of a unit lower triangular system; S enters its right side linearly, so what needs no
// S is made for all chunks side by side (`memory_pairs`): the decays, the weights e^(c_i - c_j) (q_i . k_j), and the
// system solved for write_i val_i (`u0`) and for write_i e^c_i k_i (`w`), so that w = u0 - w S. What is left goes from
// chunk to chunk (`memory_scan`): three products with S or of 64 tokens for 16 columns of S at a time. All products are
// float32 on the matrix unit (16x16x4: float32 operands, float32 sums). The sums c are taken in float64: their
// differences decide what a token far back in the chunk still weighs.
//
// The matrix unit's operands: lane l holds row (or column) l % 16 and k = l / 16; four instructions take k = 16 s +
// 4 (l / 16) + e for e = 0 .. 3, so that a lane holds four neighbours for four of them. The accumulator: column l % 16,
// rows 4 (l / 16) + e. What the first kernel leaves for the second lies in the order of those lanes (tiles of 64 lanes by
// four elements): 16 lanes that read 16 bytes each of 16 rows would ask the cache for 16 lines, four times an
// instruction. Rows are filled up with zeros to 16 NB elements on the way, and tokens beyond a run's last (in its last
// chunk) have zeros for write weights, so that what else is made of them meets zeros.
constexpr int CHUNK = 64;
constexpr int TILE = 256;                 // elements of 64 lanes by four

struct ChunkArgs {
  const float* u;           // [T, ld]
  int ld, q_at, k_at, v_at;
  const float* log_decay;   // [T, H]; [H] with decay_ld = 0; KEYED: [T, H n]
  int decay_ld;
  const float* write;       // [T, H] or null: 1
  const int* run_start;
  const int* cached;
  const int* slots;
  const int* chunk_run;     // [chunks]
  const int* chunk_begin;   // [chunks]
  int chunks;
  const int* long_run;      // [num_long]
  const int* long_first;    // [num_long]
  int num_long;
  float* memory;            // [slots, 2, H, v, n]
  float* out;               // [T, H v]
  float* gates;             // [chunks, H, 3, 64]: e^c_i, e^(c_64 - c_i), write_i
  float* qx;                // [chunks, G, 4, NB, tile]: queries, token 16 w + l % 16, elements 16 s + 4 (l / 16) ..
  float* kx;                // [chunks, G, NB, 4, tile]: keys, element 16 x + l % 16, tokens 16 s + 4 (l / 16) ..
  float* pairs;             // [chunks, H, 4, 4, tile]: e^(c_i - c_j) (q_i . k_j), i = 16 w + l % 16, j = 16 s + 4 (l / 16) ..;
                            //   zero for j > i, unwritten for s > w
  float* wx;                // [chunks, H, 4, NB, tile]: w, as the queries
  float* ux;                // [chunks, H, blocks of 16 columns, 4, tile]: u0, column l % 16, tokens 16 w + 4 (l / 16) ..
  float* keep;              // KEYED: [chunks, H, 16 NB]: e^c_64 a row of S (and qx and kx, a head's, hold the scaled ones)
  int heads, groups, n, v;
};

// A chunk's queries or keys to LDS, a token's row by row, zeros behind n.
template <int NB, int THREADS, bool ALIGNED>
__device__ __forceinline__ void stage_rows(const float* src, int ld, int len, int n, float* dst) {
  constexpr int LD = 16 * NB + 4, PT = 4 * NB;        // 16-byte pieces of a token
#pragma unroll 4
  for (int f = threadIdx.x; f < CHUNK * PT; f += THREADS) {
    const int t = f / PT, d = 4 * (f - t * PT);
    *(f32x4*)(dst + t * LD + d) = load4<ALIGNED>(src + (unsigned)(min(t, len - 1) * ld) + d, n - d);
  }
}

// grid: chunks * groups * parts of a group's heads, `per` heads a block. Wave w of the first four makes the products
// q . k of tokens 16 w .. 16 w + 15 once for the group (with DELTA wave 4 + w the products k . k), then every head's weights.
// With DELTA the system (I + M) x = b, M strictly lower triangular, is solved by blocks of 16 rows: the diagonal blocks
// are inverted (a lane a column), and x_i = T_ii (b_i - sum_{k<i} M_ik x_k) follows on the matrix unit, two blocks of 16
// columns of b a wave at a time: an accumulator's rows are just what a lane hands to the next product as its second
// operand. Dynamic LDS: queries (later w), keys, with DELTA -M and the inverted blocks.
template <int NB, bool DELTA, bool ALIGNED>
__global__ void __launch_bounds__(DELTA ? 512 : 256) memory_pairs_kernel(ChunkArgs a, int parts, int per) {
  constexpr int THREADS = DELTA ? 512 : 256, WAVES = THREADS / 64;
  constexpr int LD = 16 * NB + 4, MLD = CHUNK + 4, TLD = 20;
  extern __shared__ __attribute__((aligned(16))) float room[];
  __shared__ double cs[CHUNK];
  __shared__ __attribute__((aligned(16))) float beta[CHUNK], up[CHUNK];
  float* q_l = room;                            // [64][LD]
  float* k_l = q_l + CHUNK * LD;                // [64][LD]
  float* mn = k_l + CHUNK * LD;                 // [64][MLD]: -M, row by row
  float* td = mn + CHUNK * MLD;                 // [64][TLD]: the inverted diagonal blocks
  const int part = blockIdx.x % parts, rest = blockIdx.x / parts;
  const int group = rest % a.groups, chunk = rest / a.groups;
  const int run = a.chunk_run[chunk], begin = a.chunk_begin[chunk];
  const int t0 = a.run_start[run] + begin, len = min(CHUNK, a.run_start[run + 1] - t0);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int w4 = wave & 3;
  const bool keys_side = wave >= 4;             // (DELTA: the waves that make k . k)
  const float* base = a.u + (size_t)t0 * a.ld;
  stage_rows<NB, THREADS, ALIGNED>(base + a.q_at + group * a.n, a.ld, len, a.n, q_l);
  stage_rows<NB, THREADS, ALIGNED>(base + a.k_at + group * a.n, a.ld, len, a.n, k_l);
  __syncthreads();
  // prod[cb][e]: token j = 16 cb + 4 g + e (key) with token i = 16 w4 + r
  f32x4 prod[4];
#pragma unroll
  for (int cb = 0; cb < 4; ++cb) prod[cb] = (f32x4){0.f, 0.f, 0.f, 0.f};
  {
    const float* mine = (keys_side ? k_l : q_l) + (16 * w4 + r) * LD + 4 * g;
    float* qx = a.qx + ((size_t)(chunk * a.groups + group) * 4 + w4) * NB * TILE + 4 * lane;
#pragma unroll 2
    for (int s = 0; s < NB; ++s) {
      const f32x4 x = *(const f32x4*)(mine + 16 * s);
      if (!keys_side && part == 0) *(f32x4*)(qx + s * TILE) = x;
#pragma unroll
      for (int cb = 0; cb < 4; ++cb) {
        if (cb > w4) continue;
        const f32x4 kb = *(const f32x4*)(k_l + (16 * cb + r) * LD + 16 * s + 4 * g);
#pragma unroll
        for (int e = 0; e < 4; ++e) prod[cb] = __builtin_amdgcn_mfma_f32_16x16x4f32(kb[e], x[e], prod[cb], 0, 0, 0);
      }
    }
  }
  if (part == 0) {
    float* kx = a.kx + (size_t)(chunk * a.groups + group) * NB * 4 * TILE + 4 * lane;
    for (int f = wave; f < 4 * NB; f += WAVES) {
      const int x = f >> 2, s = f & 3;
      f32x4 v;
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = k_l[(16 * s + 4 * g + e) * LD + 16 * x + r];
      *(f32x4*)(kx + f * TILE) = v;
    }
  }
  const int per_group = a.heads / a.groups;
  for (int hh = part * per; hh < min(per_group, (part + 1) * per); ++hh) {
    const int head = group * per_group + hh;
    const size_t place = (size_t)chunk * a.heads + head;
    if (wave == 0) {
      const size_t at = (size_t)(t0 + min(lane, len - 1)) * a.heads + head;
      double c = lane < len ? (double)a.log_decay[(size_t)(t0 + min(lane, len - 1)) * a.decay_ld + head] : 0.0;
#pragma unroll
      for (int d = 1; d < 64; d *= 2) {
        const double before = __shfl_up(c, d, 64);
        if (lane >= d) c += before;
      }
      const double all = __shfl(c, 63, 64);
      const float e = expf((float)c), b = lane < len ? (a.write ? a.write[at] : 1.f) : 0.f;
      cs[lane] = c;
      up[lane] = e;
      beta[lane] = b;
      float* gates = a.gates + place * 3 * CHUNK + lane;
      gates[0] = e;
      gates[CHUNK] = expf((float)(all - c));
      gates[2 * CHUNK] = b;
    }
    __syncthreads();
    {
      const int i = 16 * w4 + r;
      const double ci = cs[i];
      const float bi = beta[i];
      float* pairs = a.pairs + (place * 4 + w4) * 4 * TILE + 4 * lane;
#pragma unroll
      for (int cb = 0; cb < 4; ++cb) {
        if (cb > w4) continue;
        f32x4 v;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int j = 16 * cb + 4 * g + e;
          const float x = prod[cb][e] * expf((float)fmin(ci - cs[j], 0.0));
          if (keys_side)
            v[e] = j < i ? -bi * x : 0.f;
          else
            v[e] = j <= i ? x : 0.f;
        }
        if (keys_side)
          *(f32x4*)(mn + i * MLD + 16 * cb + 4 * g) = v;
        else
          *(f32x4*)(pairs + cb * TILE) = v;
      }
    }
    if (DELTA) {
      __syncthreads();
      if (wave < 4) {
        // the inverse of I + M_ww: column r, x_i = [i = r] - sum_{j<i} M[i, j] x_j
        const float* m = mn + 16 * wave * MLD + 16 * wave;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          float acc = i == r ? 1.f : 0.f;
#pragma unroll
          for (int j4 = 0; j4 < (i + 3) / 4; ++j4) {
            const f32x4 row = *(const f32x4*)(m + i * MLD + 4 * j4);
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (4 * j4 + e < i) acc += row[e] * x[4 * j4 + e];
          }
          x[i] = acc;
        }
        if (g == 0) {
#pragma unroll
          for (int i = 0; i < 16; ++i) td[(16 * wave + i) * TLD + r] = x[i];
        }
      }
      __syncthreads();
      const float* vals = base + a.v_at + head * a.v;
      const int vb = (a.v + 15) / 16;
      for (int b0 = 2 * wave; b0 < vb + NB; b0 += 2 * WAVES) {      // blocks of 16 columns: the values', then the keys'
        f32x4 x[2][4];                                              // [block of columns][block of rows]
#pragma unroll
        for (int cc = 0; cc < 2; ++cc) {
          const bool value = b0 + cc < vb;
          const int c = 16 * (b0 + cc) + r, d = min(16 * (b0 + cc - vb) + r, 16 * NB - 1);
#pragma unroll
          for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const int t = 16 * i + 4 * g + e;
              if (value)
                x[cc][i][e] = vals[(unsigned)(min(t, len - 1) * a.ld) + min(c, a.v - 1)];
              else
                x[cc][i][e] = k_l[t * LD + d] * up[t];
            }
#pragma unroll
          for (int i = 0; i < 4; ++i) x[cc][i] = x[cc][i] * *(const f32x4*)(beta + 16 * i + 4 * g);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
#pragma unroll
          for (int kb = 0; kb < i; ++kb) {
            const f32x4 m = *(const f32x4*)(mn + (16 * i + r) * MLD + 16 * kb + 4 * g);
#pragma unroll
            for (int e = 0; e < 4; ++e)
#pragma unroll
              for (int cc = 0; cc < 2; ++cc) x[cc][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(m[e], x[cc][kb][e], x[cc][i], 0, 0, 0);
          }
          const f32x4 t = *(const f32x4*)(td + (16 * i + r) * TLD + 4 * g);
          f32x4 y[2];
#pragma unroll
          for (int cc = 0; cc < 2; ++cc) y[cc] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int e = 0; e < 4; ++e)
#pragma unroll
            for (int cc = 0; cc < 2; ++cc) y[cc] = __builtin_amdgcn_mfma_f32_16x16x4f32(t[e], x[cc][i][e], y[cc], 0, 0, 0);
#pragma unroll
          for (int cc = 0; cc < 2; ++cc) x[cc][i] = y[cc];
        }
#pragma unroll
        for (int cc = 0; cc < 2; ++cc) {
          if (b0 + cc < vb) {
            float* ux = a.ux + (place * vb + b0 + cc) * 4 * TILE + 4 * lane;
#pragma unroll
            for (int i = 0; i < 4; ++i) *(f32x4*)(ux + i * TILE) = x[cc][i];
          } else if (b0 + cc < vb + NB) {
            const int d = 16 * (b0 + cc - vb) + r;
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
              for (int e = 0; e < 4; ++e) q_l[(16 * i + 4 * g + e) * LD + d] = x[cc][i][e];      // (nobody reads the queries any more)
          }
        }
      }
      __syncthreads();
      float* wx = a.wx + place * 4 * NB * TILE + 4 * lane;
      for (int f = wave; f < 4 * NB; f += WAVES) {
        const int w = f / NB, s = f - w * NB;
        *(f32x4*)(wx + f * TILE) = *(const f32x4*)(q_l + (16 * w + r) * LD + 16 * s + 4 * g);
      }
    }
    __syncthreads();      // before the next head's decays
  }
}

// KEYED, a decay for every row d of S: with c_i[d] the chunk's sums,
//     o_i = sum_d q_i[d] e^(c_i[d]) S[d] + sum_{j<=i} A_ij val_j,   A_ij = sum_d q_i[d] k_j[d] e^(c_i[d] - c_j[d])
//     the state after the chunk: e^(c_64[d]) S[d] + sum_j k_j[d] e^(c_64[d] - c_j[d]) val_j
// No single point d of reference serves all of A: e^(-c_j) alone overflows where a channel forgets fast. The chunk goes in
// four blocks of 16 tokens, l the sums inside a block and L_b a block's whole: a pair of blocks J < I is the product of
// q_i e^(l_i) e^(L_(J+1) + .. + L_(I-1)) with k_j e^(L_J - l_j), no exponent above zero. Inside a block q_i e^(l_i) meets
// k_j e^(-l_j) as long as no channel of the block forgets by more than 2^-LEVEL (float32 then still holds both factors to
// full precision); a block that does makes its weights pair by pair, the exponents' difference first. Sums are taken in
// float64 and kept in powers of two.
//
// grid: chunks * heads; channels in pieces of at most 128; wave w has the tokens 16 w .. 16 w + 15 as queries.
constexpr double LOG2E = 1.4426950408889634074;
constexpr float LEVEL = 60.f;
__device__ __forceinline__ float pow2(float x) { return __builtin_amdgcn_exp2f(x); }

template <int NB, bool ALIGNED>
__global__ void __launch_bounds__(256) memory_pairs_keyed_kernel(ChunkArgs a) {
  constexpr int P = NB < 8 ? NB : 8, PIECES = NB / P, PD = 16 * P, LD = PD + 4, PT = 4 * P;
  extern __shared__ __attribute__((aligned(16))) float room[];
  __shared__ __attribute__((aligned(16))) float tot[4 * PD];      // L_b, a block of tokens behind the other
  float* q_l = room;                            // [64][LD]
  float* k_l = q_l + CHUNK * LD;                // [64][LD]
  float* c_l = k_l + CHUNK * LD;                // [64][LD]: l
  const int head = blockIdx.x % a.heads, chunk = blockIdx.x / a.heads;
  const int run = a.chunk_run[chunk], begin = a.chunk_begin[chunk];
  const int t0 = a.run_start[run] + begin, len = min(CHUNK, a.run_start[run + 1] - t0);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const size_t place = (size_t)chunk * a.heads + head;
  const float* base = a.u + (size_t)t0 * a.ld + head * a.n;
  const float* decay = a.log_decay + (size_t)t0 * a.decay_ld + head * a.n;
  // prod[cb][e]: token j = 16 cb + 4 g + e (key) with token i = 16 wave + r
  f32x4 prod[4];
#pragma unroll
  for (int cb = 0; cb < 4; ++cb) prod[cb] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int piece = 0; piece < PIECES; ++piece) {
    const int d0 = PD * piece;
    if (piece > 0) __syncthreads();             // before the next piece takes the place of what this one read
#pragma unroll 4
    for (int f = threadIdx.x; f < CHUNK * PT; f += 256) {        // zeros behind n and from the run's end on
      const int t = f / PT, d = 4 * (f - t * PT);
      const float* row = base + (unsigned)(min(t, len - 1) * a.ld) + d0 + d;
      const int valid = t < len ? a.n - d0 - d : 0;
      *(f32x4*)(q_l + t * LD + d) = load4<ALIGNED>(row + a.q_at, valid);
      *(f32x4*)(k_l + t * LD + d) = load4<ALIGNED>(row + a.k_at, valid);
    }
    for (int f = threadIdx.x; f < 4 * PD; f += 256) {
      const int b = f / PD, d = f - b * PD;
      const bool in = d0 + d < a.n;
      float got[16];
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int t = 16 * b + i;
        got[i] = in && t < len ? decay[(unsigned)(t * a.decay_ld) + d0 + d] : 0.f;
      }
      double c = 0.0;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        c += (double)got[i];
        c_l[(16 * b + i) * LD + d] = (float)(c * LOG2E);
      }
      tot[f] = (float)(c * LOG2E);
    }
    __syncthreads();
    // what the second kernel reads: q_i e^(c_i), k_j e^(c_64 - c_j), e^(c_64)
    float* qx = a.qx + (place * 4 + wave) * NB * TILE + 4 * lane;
    const float* my_q = q_l + (16 * wave + r) * LD + 4 * g;
    const float* my_c = c_l + (16 * wave + r) * LD + 4 * g;
#pragma unroll 2
    for (int s = 0; s < P; ++s) {
      const f32x4 q = *(const f32x4*)(my_q + 16 * s), l = *(const f32x4*)(my_c + 16 * s);
      f32x4 before = {0.f, 0.f, 0.f, 0.f};
      for (int b = 0; b < wave; ++b) before = before + *(const f32x4*)(tot + b * PD + 16 * s + 4 * g);
      f32x4 x;
#pragma unroll
      for (int e = 0; e < 4; ++e) x[e] = q[e] * pow2(before[e] + l[e]);
      *(f32x4*)(qx + (P * piece + s) * TILE) = x;
    }
    float* kx = a.kx + place * NB * 4 * TILE + 4 * lane;
    for (int f = wave; f < 4 * P; f += 4) {
      const int x = f >> 2, s = f & 3, d = 16 * x + r;
      float after = tot[s * PD + d];
      for (int b = s + 1; b < 4; ++b) after += tot[b * PD + d];
      f32x4 v;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int at = (16 * s + 4 * g + e) * LD + d;
        v[e] = k_l[at] * pow2(after - c_l[at]);
      }
      *(f32x4*)(kx + (4 * P * piece + f) * TILE) = v;
    }
    for (int d = threadIdx.x; d < PD; d += 256)
      a.keep[place * 16 * NB + d0 + d] = pow2(tot[d] + tot[PD + d] + tot[2 * PD + d] + tot[3 * PD + d]);
    // the weights: does a channel of this wave's block forget too fast for one point of reference?
    float worst = 0.f;
    for (int d = lane; d < PD; d += 64) worst = fmaxf(worst, -tot[wave * PD + d]);
    const bool gentle = wave_max(worst) <= LEVEL;
#pragma unroll 2
    for (int s = 0; s < P; ++s) {
      const f32x4 q = *(const f32x4*)(my_q + 16 * s), l = *(const f32x4*)(my_c + 16 * s);
      f32x4 x;                                   // q_i e^(l_i), times the blocks between as they come in between
#pragma unroll
      for (int e = 0; e < 4; ++e) x[e] = q[e] * pow2(l[e]);
      if (gentle) {
        f32x4 kb = *(const f32x4*)(k_l + (16 * wave + r) * LD + 16 * s + 4 * g);
#pragma unroll
        for (int e = 0; e < 4; ++e) kb[e] *= pow2(-l[e]);
#pragma unroll
        for (int cb = 0; cb < 4; ++cb)
          if (cb == wave) {
#pragma unroll
            for (int e = 0; e < 4; ++e) prod[cb] = __builtin_amdgcn_mfma_f32_16x16x4f32(kb[e], x[e], prod[cb], 0, 0, 0);
          }
      }
#pragma unroll
      for (int cb = 2; cb >= 0; --cb) {
        if (cb >= wave) continue;
        const f32x4 whole = *(const f32x4*)(tot + cb * PD + 16 * s + 4 * g);
        f32x4 kb = *(const f32x4*)(k_l + (16 * cb + r) * LD + 16 * s + 4 * g);
        const f32x4 lk = *(const f32x4*)(c_l + (16 * cb + r) * LD + 16 * s + 4 * g);
#pragma unroll
        for (int e = 0; e < 4; ++e) kb[e] *= pow2(whole[e] - lk[e]);
#pragma unroll
        for (int e = 0; e < 4; ++e) prod[cb] = __builtin_amdgcn_mfma_f32_16x16x4f32(kb[e], x[e], prod[cb], 0, 0, 0);
#pragma unroll
        for (int e = 0; e < 4; ++e) x[e] *= pow2(whole[e]);
      }
    }
    if (!gentle) {
      // pair by pair: the lane's query i = 16 wave + r with the keys 16 wave + 4 g + e
      f32x4 sum = {0.f, 0.f, 0.f, 0.f};
      const float* qi = q_l + (16 * wave + r) * LD;
      const float* ci = c_l + (16 * wave + r) * LD;
      for (int d = 0; d < PD; d += 4) {
        const f32x4 q = *(const f32x4*)(qi + d), l = *(const f32x4*)(ci + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const f32x4 k = *(const f32x4*)(k_l + (16 * wave + 4 * g + e) * LD + d);
          const f32x4 lk = *(const f32x4*)(c_l + (16 * wave + 4 * g + e) * LD + d);
#pragma unroll
          for (int c = 0; c < 4; ++c) sum[e] += q[c] * k[c] * pow2(fminf(l[c] - lk[c], 0.f));
        }
      }
#pragma unroll
      for (int cb = 0; cb < 4; ++cb)
        if (cb == wave) prod[cb] = prod[cb] + sum;
    }
  }
  float* pairs = a.pairs + (place * 4 + wave) * 4 * TILE + 4 * lane;
#pragma unroll
  for (int cb = 0; cb < 4; ++cb) {
    if (cb > wave) continue;
    f32x4 v;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = 16 * cb + 4 * g + e <= 16 * wave + r ? prod[cb][e] : 0.f;
    *(f32x4*)(pairs + cb * TILE) = v;
  }
}

// grid: (run, head) pairs in eights * column blocks: the blocks of a (run, head) come eight apart, so that they share an
// XCD's cache. A block walks a run's chunks for 16 columns of S; wave w has the chunk's tokens 16 w .. 16 w + 15, and of S
// the blocks of 16 rows w, w + 4, ..., in the accumulators from chunk to chunk. What a chunk's products read of memory is
// asked for two chunks ahead, into the registers (one set for even, one for odd chunks) that the chunk before last has
// just read: a compute unit has one such block, and a load takes as long as a chunk's products do.
template <int NB, int MODE, bool ALIGNED>
__global__ void __launch_bounds__(256, 1) memory_scan_kernel(ChunkArgs a, int column_blocks) {
  constexpr bool DELTA = MODE == DELTA_RULE;
  constexpr int RB = (NB + 3) / 4;               // blocks of rows of S a wave
  constexpr int SLD = 16 * NB + 4, ULD = CHUNK + 4;
  __shared__ __attribute__((aligned(16))) float s_l[16 * SLD];        // [column][row]
  __shared__ __attribute__((aligned(16))) float u_l[16 * ULD];        // [column][token]: the writes
  __shared__ __attribute__((aligned(16))) float b_l[MODE == KEYED ? 4 : 16 * ULD];        // the same times e^(c_64 - c_j)
  const int rh = (blockIdx.x & 7) + 8 * (blockIdx.x / (8 * column_blocks));
  const int cb = (blockIdx.x >> 3) % column_blocks;
  if (rh >= a.num_long * a.heads) return;
  const int li = rh / a.heads, head = rh - li * a.heads, group = head / (a.heads / a.groups);
  const int run = a.long_run[li], first = a.long_first[li];
  const int start = a.run_start[run], count = a.run_start[run + 1] - start, have = a.cached[run], slot = a.slots[run];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int col = 16 * cb + r;
  const bool col_ok = col < a.v;
  const int ccol = col_ok ? col : 0;
  const int from = (have - 1) & 1, to = (have + count - 1) & 1;
  const size_t head_at = (size_t)slot * 2 * a.heads + head;
  const f32x4 zero4 = {0.f, 0.f, 0.f, 0.f};
  f32x4 S[RB];                                   // (rows from n on stay zero: the keys have zeros there)
  auto share = [&]() {
#pragma unroll
    for (int x = 0; x < RB; ++x)
      if (wave + 4 * x < NB) *(f32x4*)(s_l + r * SLD + 16 * (wave + 4 * x) + 4 * g) = S[x];
  };
#pragma unroll
  for (int x = 0; x < RB; ++x) {
    const int row = 16 * (wave + 4 * x) + 4 * g;
    const float* p = a.memory + ((head_at + (size_t)from * a.heads) * a.v + ccol) * a.n + row;
    S[x] = load4<ALIGNED>(p, have > 0 && col_ok ? a.n - row : 0);
  }
  share();
  struct Set {
    f32x4 wa[DELTA ? NB : 1], qa[NB], pa[4], kt[RB][4], keep[MODE == KEYED ? RB : 1], u0, up, down, wr;
    float decay;
  };
  Set even, odd;
  auto fetch_state_side = [&](int c, Set& z) {          // what meets S: this wave's tokens' queries and rows of w, their u0
    const int t0 = start + CHUNK * c, len = min(CHUNK, count - CHUNK * c);
    const size_t of_group = (size_t)(first + c) * a.groups + group, of_head = (size_t)(first + c) * a.heads + head;
    const float* q = a.qx + (of_group * 4 + wave) * NB * TILE + 4 * lane;
    const float* w = a.wx + (of_head * 4 + wave) * NB * TILE + 4 * lane;
#pragma unroll
    for (int s = 0; s < NB; ++s) {
      z.qa[s] = *(const f32x4*)(q + s * TILE);
      if (DELTA) z.wa[DELTA ? s : 0] = *(const f32x4*)(w + s * TILE);
    }
    if (DELTA) {
      z.u0 = *(const f32x4*)(a.ux + ((of_head * column_blocks + cb) * 4 + wave) * TILE + 4 * lane);
    } else {
      const float* vals = a.u + (size_t)t0 * a.ld + a.v_at + head * a.v + ccol;
#pragma unroll
      for (int e = 0; e < 4; ++e) z.u0[e] = vals[(unsigned)(min(16 * wave + 4 * g + e, len - 1) * a.ld)];
    }
    if (MODE == KEYED) {
#pragma unroll
      for (int x = 0; x < RB; ++x)
        z.keep[MODE == KEYED ? x : 0] = *(const f32x4*)(a.keep + of_head * 16 * NB + 16 * min(wave + 4 * x, NB - 1) + 4 * g);
      return;
    }
    const float* gates = a.gates + of_head * 3 * CHUNK;
    z.up = *(const f32x4*)(gates + 16 * wave + 4 * g);
    z.down = *(const f32x4*)(gates + CHUNK + 16 * wave + 4 * g);
    if (!DELTA) z.wr = *(const f32x4*)(gates + 2 * CHUNK + 16 * wave + 4 * g);
    z.decay = gates[CHUNK - 1];
  };
  auto fetch_token_side = [&](int c, Set& z) {          // what meets the writes: the weights among the tokens, the keys
    const float* pairs = a.pairs + (((size_t)(first + c) * a.heads + head) * 4 + wave) * 4 * TILE + 4 * lane;
    const float* k = a.kx + ((size_t)(first + c) * a.groups + group) * NB * 4 * TILE + 4 * lane;
#pragma unroll
    for (int s = 0; s < 4; ++s) z.pa[s] = *(const f32x4*)(pairs + min(s, wave) * TILE);
#pragma unroll
    for (int x = 0; x < RB; ++x)
#pragma unroll
      for (int s = 0; s < 4; ++s) z.kt[x][s] = *(const f32x4*)(k + (4 * min(wave + 4 * x, NB - 1) + s) * TILE);
  };
  const int chunks = (count + CHUNK - 1) / CHUNK;
  fetch_state_side(0, even);
  fetch_token_side(0, even);
  if (chunks > 1) {
    fetch_state_side(1, odd);
    fetch_token_side(1, odd);
  }
  __syncthreads();
  auto chunk = [&](int c, Set& z) {
    const int t0 = start + CHUNK * c, len = min(CHUNK, count - CHUNK * c);
    f32x4 o = zero4, m = zero4;
#pragma unroll
    for (int s = 0; s < NB; ++s) {
      const f32x4 s4 = *(const f32x4*)(s_l + r * SLD + 16 * s + 4 * g);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        o = __builtin_amdgcn_mfma_f32_16x16x4f32(z.qa[s][e], s4[e], o, 0, 0, 0);
        if (DELTA) m = __builtin_amdgcn_mfma_f32_16x16x4f32(z.wa[DELTA ? s : 0][e], s4[e], m, 0, 0, 0);
      }
    }
    // (KEYED: the decays are in the queries, the keys and the weights already)
    const f32x4 u4 = DELTA ? z.u0 - m : MODE == KEYED ? z.u0 : z.wr * z.u0;
    *(f32x4*)(u_l + r * ULD + 16 * wave + 4 * g) = u4;
    if (MODE != KEYED) {
      *(f32x4*)(b_l + r * ULD + 16 * wave + 4 * g) = u4 * z.down;
      o = o * z.up;
    }
#pragma unroll
    for (int x = 0; x < RB; ++x) {
      if (MODE == KEYED)
        S[x] = S[x] * z.keep[MODE == KEYED ? x : 0];
      else
        S[x] = S[x] * z.decay;
    }
    if (c + 2 < chunks) fetch_state_side(c + 2, z);
    __syncthreads();
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const f32x4 us = *(const f32x4*)(u_l + r * ULD + 16 * s + 4 * g);
      const f32x4 bs = MODE == KEYED ? us : *(const f32x4*)(b_l + r * ULD + 16 * s + 4 * g);
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int x = 0; x < RB; ++x) S[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(z.kt[x][s][e], bs[e], S[x], 0, 0, 0);
      if (s <= wave) {
#pragma unroll
        for (int e = 0; e < 4; ++e) o = __builtin_amdgcn_mfma_f32_16x16x4f32(z.pa[s][e], us[e], o, 0, 0, 0);
      }
    }
    if (c + 2 < chunks) fetch_token_side(c + 2, z);
    share();
    float* out = a.out + ((size_t)t0 * a.heads + head) * a.v + ccol;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = 16 * wave + 4 * g + e;
      if (i < len && col_ok) out[(unsigned)(i * a.heads * a.v)] = o[e];
    }
    __syncthreads();
  };
  for (int c = 0; c < chunks; c += 2) {
    chunk(c, even);
    if (c + 1 < chunks) chunk(c + 1, odd);
  }
  if (!col_ok) return;
#pragma unroll
  for (int x = 0; x < RB; ++x) {
    const int row = 16 * (wave + 4 * x) + 4 * g;
    float* p = a.memory + ((head_at + (size_t)to * a.heads) * a.v + col) * a.n + row;
    if (ALIGNED) {
      if (row < a.n) *(f32x4*)p = S[x];
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (row + e < a.n) p[e] = S[x][e];
    }
  }
}

template <int NB, int MODE, bool ALIGNED>
int launch_chunks(const ChunkArgs& a, hipStream_t stream) {
  constexpr bool DELTA = MODE == DELTA_RULE;
  const int per_group = a.heads / a.groups;
  const int column_blocks = (a.v + 15) / 16;
  static bool configured = false;
  if constexpr (MODE == KEYED) {
    constexpr int lds = 3 * CHUNK * (16 * (NB < 8 ? NB : 8) + 4) * (int)sizeof(float);
    if (!configured) {
      const hipError_t e = hipFuncSetAttribute((const void*)memory_pairs_keyed_kernel<NB, ALIGNED>,
                                               hipFuncAttributeMaxDynamicSharedMemorySize, lds);
      TNX_REQUIRE(e == hipSuccess, "memory_chunks: cannot reserve %d bytes of LDS: %s", lds, hipGetErrorString(e));
      configured = true;
    }
    memory_pairs_keyed_kernel<NB, ALIGNED><<<(unsigned)((size_t)a.chunks * a.heads), 256, lds, stream>>>(a);
  } else {
    int per = 1;                                   // heads of a group a block of the first kernel
    while (!DELTA && per < per_group && (long long)a.chunks * a.groups * ((per_group + 2 * per - 1) / (2 * per)) >= 2 * tnx_compute_units())
      per *= 2;
    const int parts = (per_group + per - 1) / per;
    const int lds = (2 * CHUNK * (16 * NB + 4) + (DELTA ? CHUNK * (CHUNK + 4) + CHUNK * 20 : 0)) * (int)sizeof(float);
    if (!configured) {
      const hipError_t e = hipFuncSetAttribute((const void*)memory_pairs_kernel<NB, DELTA, ALIGNED>,
                                               hipFuncAttributeMaxDynamicSharedMemorySize, lds);
      TNX_REQUIRE(e == hipSuccess, "memory_chunks: cannot reserve %d bytes of LDS: %s", lds, hipGetErrorString(e));
      configured = true;
    }
    memory_pairs_kernel<NB, DELTA, ALIGNED>
        <<<(unsigned)((size_t)a.chunks * a.groups * parts), DELTA ? 512 : 256, lds, stream>>>(a, parts, per);
  }
  TNX_CHECK_LAUNCH("memory_pairs");
  memory_scan_kernel<NB, MODE, ALIGNED>
      <<<(unsigned)((a.num_long * a.heads + 7) / 8 * 8 * column_blocks), 256, 0, stream>>>(a, column_blocks);
  TNX_CHECK_LAUNCH("memory_scan");
  return 0;
}

template <int MODE, bool ALIGNED>
int launch_chunks_sized(const ChunkArgs& a, int nb, hipStream_t stream) {
  switch (nb) {
    case 2: return launch_chunks<2, MODE, ALIGNED>(a, stream);
    case 4: return launch_chunks<4, MODE, ALIGNED>(a, stream);
    case 8: return launch_chunks<8, MODE, ALIGNED>(a, stream);
    default: return launch_chunks<16, MODE, ALIGNED>(a, stream);
  }
}

// ------------------------------------------------------------------------------------------ after the memory

struct FinishArgs {
  const float* o;           // [T, width]
  const float* gate;        // [T, gate_ld]
  long long gate_ld;
  const float* weight;      // [width] or null: 1
  float eps;
  int parts, gate_first;
  const float* skip;        // [heads] or null
  const float* x;           // [T, x_ld]
  long long x_ld;
  int per_head;             // elements a head
  void* out;                // [T, out_ld]
  long long out_ld;
  float out_scale;
  int tokens, width;
};

// A row's `parts` equal parts at unit root mean square, times weight; (o + skip x) silu(gate) before the norm or
// silu(gate) after it. A part is THREADS threads' work, four neighbours a thread at a time (ALIGNED: 16-byte loads; parts,
// rows and heads begin at multiples of four elements). HELD pieces of a part stay in registers between the two passes.
template <typename T, int THREADS, bool ALIGNED>
__global__ void __launch_bounds__(256) gated_norm_kernel(FinishArgs a) {
  __shared__ float scratch[4];
  constexpr int PER_BLOCK = 256 / THREADS;
  const long long idx = (long long)blockIdx.x * PER_BLOCK + (THREADS == 256 ? 0 : threadIdx.x / THREADS);
  const bool active = idx < (long long)a.tokens * a.parts;
  if (THREADS == 64 && !active) return;
  const size_t t = active ? idx / a.parts : 0;
  const int part = active ? (int)(idx - (long long)t * a.parts) : 0;
  const int size = a.width / a.parts, first = part * size;
  const int me = threadIdx.x % THREADS;
  const float* o = a.o + t * a.width + first;
  const float* gate = a.gate + t * a.gate_ld + first;
  const float* x = a.skip ? a.x + t * a.x_ld + first : nullptr;
  auto value = [&](int i) {            // elements i .. i + 3, zeros from the part's end on
    f32x4 y = load4<ALIGNED>(o + i, size - i);
    if (x) {
      const f32x4 xs = load4<ALIGNED>(x + i, size - i);
      if (ALIGNED) {
        y = y + a.skip[(first + i) / a.per_head] * xs;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (i + e < size) y[e] += a.skip[(first + i + e) / a.per_head] * xs[e];
      }
    }
    if (a.gate_first) {
      const f32x4 gs = load4<ALIGNED>(gate + i, size - i);
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] *= silu(gs[e]);
    }
    return y;
  };
  constexpr int HELD = 2;
  f32x4 held[HELD];
  float s = 0.f;
#pragma unroll
  for (int c = 0; c < HELD; ++c) {
    const int i = 4 * (me + THREADS * c);
    held[c] = i < size ? value(i) : (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) s += held[c][e] * held[c][e];
  }
  for (int i = 4 * (me + THREADS * HELD); i < size; i += 4 * THREADS) {
    const f32x4 y = value(i);
#pragma unroll
    for (int e = 0; e < 4; ++e) s += y[e] * y[e];
  }
  if (THREADS == 256) {
    s = block_sum<4>(s, scratch);
  } else {
    s = sum16(s);
    if (THREADS >= 32) {
      unsigned lo, hi;
      swap_rows(__float_as_uint(s), lo, hi);
      s = __uint_as_float(lo) + __uint_as_float(hi);
    }
    if (THREADS >= 64) {
      unsigned lo, hi;
      swap_halves(__float_as_uint(s), lo, hi);
      s = __uint_as_float(lo) + __uint_as_float(hi);
    }
  }
  if (!active) return;
  const float r = 1.f / sqrtf(s / (float)size + a.eps);
  T* out = (T*)a.out + t * a.out_ld + first;
  auto put = [&](int i, f32x4 y) {
    y = y * r;
    if (a.weight) y = y * load4<ALIGNED>(a.weight + first + i, size - i);
    if (!a.gate_first) {
      const f32x4 gs = load4<ALIGNED>(gate + i, size - i);
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] *= silu(gs[e]);
    }
    typedef T four __attribute__((ext_vector_type(4)));
    four v;
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = from_f32<T>(y[e] * a.out_scale);
    if (ALIGNED) {
      *(four*)(out + i) = v;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (i + e < size) out[i + e] = v[e];
    }
  };
#pragma unroll
  for (int c = 0; c < HELD; ++c) {
    const int i = 4 * (me + THREADS * c);
    if (i < size) put(i, held[c]);
  }
  for (int i = 4 * (me + THREADS * HELD); i < size; i += 4 * THREADS) put(i, value(i));
}

template <typename T, bool ALIGNED>
void launch_gated_norm(const FinishArgs& a, hipStream_t stream) {
  const int size = a.width / a.parts;
  const long long rows = (long long)a.tokens * a.parts;
  if (size <= 64)
    gated_norm_kernel<T, 16, ALIGNED><<<(unsigned)((rows + 15) / 16), 256, 0, stream>>>(a);
  else if (size <= 128)
    gated_norm_kernel<T, 32, ALIGNED><<<(unsigned)((rows + 7) / 8), 256, 0, stream>>>(a);
  else if (size <= 512)
    gated_norm_kernel<T, 64, ALIGNED><<<(unsigned)((rows + 3) / 4), 256, 0, stream>>>(a);
  else
    gated_norm_kernel<T, 256, ALIGNED><<<(unsigned)rows, 256, 0, stream>>>(a);
}

}  // namespace

extern "C" int tnx_memory_inputs(const float* proj, int ld, int conv_at, int channels, const float* w, const float* bias,
                                 float* state, int taps, const int* positions, const int* token_request,
                                 const int* run_start, const int* slots, int unit_size, int unit_count, int scaled,
                                 float scale, float* u, int u_ld, int heads, int dt_at, int write_at, const float* rate,
                                 const float* dt_bias, float* log_decay, float* write, int tokens, int runs,
                                 hipStream_t stream) {
  TNX_REQUIRE(tokens >= 0 && runs >= 0 && channels > 0 && taps >= 1 && heads > 0, "memory_inputs: bad sizes");
  TNX_REQUIRE(conv_at >= 0 && ld >= conv_at + channels && dt_at >= 0 && ld >= dt_at + heads && ld >= write_at + heads,
              "memory_inputs: rows of %d elements do not hold what is read", ld);
  TNX_REQUIRE(u_ld >= channels, "memory_inputs: result rows of %d elements, %d needed", u_ld, channels);
  TNX_REQUIRE(taps == 1 || state, "memory_inputs: %d taps need the requests' state", taps);
  TNX_REQUIRE(unit_count >= 0 && unit_count <= channels && scaled <= channels &&
                  (unit_count == 0 || (unit_size > 0 && unit_size <= 256 && unit_count % unit_size == 0)),
              "memory_inputs: %d channels in unit heads of %d (up to 256 elements)", unit_count, unit_size);
  TNX_REQUIRE(runs < 65536, "memory_inputs: too many runs");
  if (tokens == 0 || runs == 0) return 0;
  const bool singles = tokens == runs;
  InputArgs a{proj, ld, conv_at, channels, w, bias, taps > 1 ? state : nullptr, taps, positions, token_request, run_start, slots,
              unit_count ? unit_size : 0, unit_count, scaled, scale, u, u_ld, heads, dt_at, write_at, rate, dt_bias, log_decay, write,
              tokens, singles};
  int lanes = 0;
  if (unit_count == 0 || unit_size == 64)
    lanes = 16;
  else if (unit_size == 128)
    lanes = 32;
  else if (unit_size == 256)
    lanes = 64;
  const int pieces = lanes ? (channels + 255) / 256 : unit_count / unit_size + (channels - unit_count + 255) / 256;
  const int gates = (heads + 63) / 64;
  // tokens a wave: as many as leave the chip a few waves a compute unit, up to 16
  int per = 1;
  while (per < 16 && (long long)(pieces + gates) * (tokens / (2 * per)) >= 8 * tnx_compute_units()) per *= 2;
  const long long rows = (tokens + per - 1) / per;
  TNX_REQUIRE(rows < 65536, "memory_inputs: too many tokens");
  const dim3 grid((pieces + gates + 3) / 4, (unsigned)rows);
#define INPUTS_LAUNCH(L, N) memory_inputs_kernel<L, N><<<grid, 256, 0, stream>>>(a, pieces, per)
#define INPUTS_TAPS(L)                        \
  if (taps == 1) INPUTS_LAUNCH(L, 1);         \
  else if (taps == 2) INPUTS_LAUNCH(L, 2);    \
  else if (taps == 3) INPUTS_LAUNCH(L, 3);    \
  else if (taps == 4) INPUTS_LAUNCH(L, 4);    \
  else INPUTS_LAUNCH(L, 0)
  if (lanes == 16) {
    INPUTS_TAPS(16);
  } else if (lanes == 32) {
    INPUTS_TAPS(32);
  } else if (lanes == 64) {
    INPUTS_TAPS(64);
  } else {
    INPUTS_TAPS(0);
  }
#undef INPUTS_TAPS
#undef INPUTS_LAUNCH
  TNX_CHECK_LAUNCH("memory_inputs");
  if (taps > 1 && !singles) {
    memory_state_kernel<<<dim3((channels + 255) / 256, runs), 256, 0, stream>>>(a);
    TNX_CHECK_LAUNCH("memory_state");
  }
  return 0;
}

extern "C" int tnx_channel_decays(const float* low, long long low_ld, const void* w, int w_dtype, const float* bias, float over_tau,
                                  float* out, int tokens, int channels, int rank, hipStream_t stream) {
  TNX_REQUIRE(tokens >= 0 && channels > 0 && rank > 0 && low_ld >= rank, "channel_decays: bad sizes");
  TNX_REQUIRE(w_dtype == TNX_F32 || w_dtype == TNX_BF16, "channel_decays: dtype %d", w_dtype);
  TNX_REQUIRE(tokens < 16 * 65535, "channel_decays: too many tokens");
  TNX_REQUIRE((uintptr_t)w % 32 == 0, "channel_decays: the matrix does not begin at a multiple of 32 bytes");
  if (tokens == 0) return 0;
  DecayArgs a{low, low_ld, w, bias, over_tau, out, tokens, channels, rank};
  const int blocks = (channels + 255) / 256;
  // few tokens: one a block, so that the chip has something to do
  if ((long long)blocks * tokens <= 4 * tnx_compute_units()) {
    if (w_dtype == TNX_F32)
      channel_decays_kernel<float, 1><<<dim3(blocks, tokens), 256, 0, stream>>>(a);
    else
      channel_decays_kernel<bf16_t, 1><<<dim3(blocks, tokens), 256, 0, stream>>>(a);
  } else {
    if (w_dtype == TNX_F32)
      channel_decays_kernel<float, 16><<<dim3(blocks, (tokens + 15) / 16), 256, 0, stream>>>(a);
    else
      channel_decays_kernel<bf16_t, 16><<<dim3(blocks, (tokens + 15) / 16), 256, 0, stream>>>(a);
  }
  TNX_CHECK_LAUNCH("channel_decays");
  return 0;
}

extern "C" int tnx_turn_heads(float* x, int ld, int at, int heads, int n, const float* freqs, int half, int interleaved,
                              const int* positions, int tokens, hipStream_t stream) {
  TNX_REQUIRE(tokens >= 0 && heads > 0 && n > 0 && at >= 0 && ld >= at + heads * n, "turn_heads: bad sizes");
  TNX_REQUIRE(half > 0 && half <= 128 && 2 * half <= n, "turn_heads: %d turned elements in heads of %d", 2 * half, n);
  if (tokens == 0) return 0;
  turn_heads_kernel<<<tokens, 256, 0, stream>>>(x, ld, at, heads, n, freqs, half, interleaved, positions);
  TNX_CHECK_LAUNCH("turn_heads");
  return 0;
}

// `mode`: 0 plain, 1 with the delta rule, 2 a decay for every row of S (`log_decay` [T, H n]). `decay_ld`: elements from one
// token's decays to the next's (0: the same for every token).
extern "C" int tnx_memory_walk(const float* u, int ld, int q_at, int k_at, int v_at, const float* log_decay, int decay_ld,
                               const float* write, const int* run_start, const int* cached, const int* slots, float* memory,
                               float* out, int tokens, int requests, int heads, int groups, int n, int v, int mode,
                               int longest, hipStream_t stream) {
  TNX_REQUIRE(mode >= PLAIN && mode <= KEYED && (mode != KEYED || (groups == heads && !write)), "memory_walk: bad mode");
  TNX_REQUIRE(decay_ld == 0 || decay_ld >= (mode == KEYED ? heads * n : heads), "memory_walk: rows of %d decays", decay_ld);
  TNX_REQUIRE(tokens >= 0 && requests >= 0 && heads > 0 && groups > 0 && heads % groups == 0 && n > 0 && v > 0,
              "memory_walk: bad sizes");
  TNX_REQUIRE(n <= 256, "memory_walk: query/key heads of up to 256 elements, got %d", n);
  TNX_REQUIRE(q_at >= 0 && k_at >= 0 && v_at >= 0 && ld >= q_at + groups * n && ld >= k_at + groups * n && ld >= v_at + heads * v,
              "memory_walk: rows of %d elements do not hold what is read", ld);
  if (tokens == 0 || requests == 0) return 0;
  TNX_REQUIRE((long long)requests * heads * ((v + 15) / 16) < (1ll << 31), "memory_walk: too many blocks");
  WalkArgs a{u, ld, q_at, k_at, v_at, log_decay, decay_ld, write, run_start, cached, slots, memory, out, heads, groups, n, v, longest};
  // rows and heads that begin at multiples of 16 bytes are loaded 16 bytes at a time
  const bool aligned = n % 4 == 0 && v % 4 == 0 && ((ld | q_at | k_at | v_at) & 3) == 0 && (uintptr_t)u % 16 == 0 &&
                       (mode != KEYED || (decay_ld % 4 == 0 && (uintptr_t)log_decay % 16 == 0));
  if (mode == DELTA_RULE)
    launch_walk_sized<DELTA_RULE>(a, requests, tokens == requests, aligned, stream);
  else if (mode == KEYED)
    launch_walk_sized<KEYED>(a, requests, tokens == requests, aligned, stream);
  else
    launch_walk_sized<PLAIN>(a, requests, tokens == requests, aligned, stream);
  TNX_CHECK_LAUNCH("memory_walk");
  return 0;
}

// The runs of several tokens that `long_run` names, chunk by chunk: `chunk_run` and `chunk_begin` name the chunks of 64
// tokens, a run's chunks one behind the other from `long_first` on. `room`: what the first kernel leaves for the second,
// `room_size` floats: with nb = 2, 4, 8 or 16, the least with n <= 16 nb, for every chunk 2 G 1024 nb + H (3 * 64 + 4096),
// and with the delta rule H (1024 nb + 1024 ceil(v / 16)) more, with a decay for every row of S H 16 nb more. `mode` and
// `decay_ld` as above.
extern "C" int tnx_memory_chunks(const float* u, int ld, int q_at, int k_at, int v_at, const float* log_decay, int decay_ld,
                                 const float* write, const int* run_start, const int* cached, const int* slots,
                                 const int* chunk_run, const int* chunk_begin, int chunks, int chunk_size, const int* long_run,
                                 const int* long_first, int num_long, float* memory, float* out, float* room,
                                 long long room_size, int heads, int groups, int n, int v, int mode, hipStream_t stream) {
  TNX_REQUIRE(mode >= PLAIN && mode <= KEYED && (mode != KEYED || (groups == heads && !write)), "memory_chunks: bad mode");
  TNX_REQUIRE(decay_ld == 0 || decay_ld >= (mode == KEYED ? heads * n : heads), "memory_chunks: rows of %d decays", decay_ld);
  TNX_REQUIRE((long long)CHUNK * decay_ld < (1ll << 31), "memory_chunks: rows too long");
  TNX_REQUIRE(heads > 0 && groups > 0 && heads % groups == 0 && n > 0 && v > 0 && n <= 256, "memory_chunks: bad sizes");
  TNX_REQUIRE(chunk_size == CHUNK, "memory_chunks: chunks of %d tokens, the kernels take %d", chunk_size, CHUNK);
  TNX_REQUIRE(q_at >= 0 && k_at >= 0 && v_at >= 0 && ld >= q_at + groups * n && ld >= k_at + groups * n && ld >= v_at + heads * v,
              "memory_chunks: rows of %d elements do not hold what is read", ld);
  if (chunks <= 0 || num_long <= 0) return 0;
  TNX_REQUIRE((long long)chunks * heads < (1ll << 30) && ((long long)num_long * heads + 7) * ((v + 15) / 16) < (1ll << 31),
              "memory_chunks: too many blocks");
  TNX_REQUIRE((long long)CHUNK * ld < (1ll << 31) && (long long)CHUNK * heads * v < (1ll << 31), "memory_chunks: rows too long");
  const int nb = n <= 32 ? 2 : n <= 64 ? 4 : n <= 128 ? 8 : 16, vb = (v + 15) / 16;
  ChunkArgs a{u, ld, q_at, k_at, v_at, log_decay, decay_ld, write, run_start, cached, slots, chunk_run, chunk_begin, chunks,
              long_run, long_first, num_long, memory, out, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr, heads,
              groups, n, v};
  const size_t of_group = (size_t)chunks * groups, of_head = (size_t)chunks * heads;
  float* at = room;
  a.qx = at, at += of_group * 4 * nb * TILE;
  a.kx = at, at += of_group * 4 * nb * TILE;
  a.pairs = at, at += of_head * 16 * TILE;
  a.gates = at, at += of_head * 3 * CHUNK;
  if (mode == KEYED) a.keep = at, at += of_head * 16 * nb;
  if (mode == DELTA_RULE) {
    a.wx = at, at += of_head * 4 * nb * TILE;
    a.ux = at, at += of_head * vb * 4 * TILE;
  }
  TNX_REQUIRE(room && (uintptr_t)room % 16 == 0 && at - room <= room_size, "memory_chunks: %lld floats of room, %lld needed",
              room_size, (long long)(at - room));
  const bool aligned = n % 4 == 0 && ((ld | q_at | k_at) & 3) == 0 && (uintptr_t)u % 16 == 0;
  if (mode == DELTA_RULE)
    return aligned ? launch_chunks_sized<DELTA_RULE, true>(a, nb, stream) : launch_chunks_sized<DELTA_RULE, false>(a, nb, stream);
  if (mode == KEYED)
    return aligned ? launch_chunks_sized<KEYED, true>(a, nb, stream) : launch_chunks_sized<KEYED, false>(a, nb, stream);
  return aligned ? launch_chunks_sized<PLAIN, true>(a, nb, stream) : launch_chunks_sized<PLAIN, false>(a, nb, stream);
}

extern "C" int tnx_gated_norm(const float* o, const float* gate, long long gate_ld, const float* weight, float eps, int parts,
                              int gate_first, const float* skip, int skip_heads, const float* x, long long x_ld, void* out,
                              long long out_ld, float out_scale, int dtype, int tokens, int width, hipStream_t stream) {
  TNX_REQUIRE(tokens >= 0 && width > 0 && parts > 0 && width % parts == 0 && gate_ld >= width && out_ld >= width,
              "gated_norm: bad sizes");
  TNX_REQUIRE(!skip || (skip_heads > 0 && width % skip_heads == 0 && x && x_ld >= width), "gated_norm: bad skip");
  TNX_REQUIRE(dtype == TNX_F32 || dtype == TNX_BF16, "gated_norm: dtype %d", dtype);
  TNX_REQUIRE((long long)tokens * parts < (1ll << 31), "gated_norm: too many rows");
  if (tokens == 0) return 0;
  FinishArgs a{o, gate, gate_ld, weight, eps, parts, gate_first, skip, x, x_ld, skip ? width / skip_heads : 1, out, out_ld, out_scale,
               tokens, width};
  const bool aligned = (width / parts) % 4 == 0 && gate_ld % 4 == 0 && (uintptr_t)gate % 16 == 0 && (uintptr_t)o % 16 == 0 &&
                       (uintptr_t)weight % 16 == 0 && (uintptr_t)out % (dtype == TNX_F32 ? 16 : 8) == 0 && out_ld % 4 == 0 &&
                       (!skip || (x_ld % 4 == 0 && a.per_head % 4 == 0 && (uintptr_t)x % 16 == 0));
  if (dtype == TNX_F32) {
    if (aligned)
      launch_gated_norm<float, true>(a, stream);
    else
      launch_gated_norm<float, false>(a, stream);
  } else if (aligned) {
    launch_gated_norm<bf16_t, true>(a, stream);
  } else {
    launch_gated_norm<bf16_t, false>(a, stream);
  }
  TNX_CHECK_LAUNCH("gated_norm");
  return 0;
}
