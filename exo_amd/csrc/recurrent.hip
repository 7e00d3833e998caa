// Recurrent mixers of layer-list decoders.  Per head, over a sequence, with S (keys x values) from zero:
//     S <- diag(a_t) S + k_t v_t^T,     o_t = S^T q_t
// Options, each a parameter of the layer: the decay per key channel (a low-rank product's output through
// a logarithm of the sigmoid) or per head (exp(-a dt), values scaled by dt), queries and keys per head or
// shared by a group of heads, a skip o_t += D v_t, a causal convolution per channel with silu in front
// of queries, keys and values.  Decays, step sizes, states and their products are float32; where a
// float32 factor enters a bf16 matrix product it goes in as two bf16 terms (value and remainder).
//
// A cache row owns a state slot (map: row -> slot): the states, and a ring of the convolution's latest
// `taps` inputs in which position p sits at p % taps - the entry a step writes is none that it reads.  A
// sequence at position 0 starts from zero whatever its slot holds.
//
// Single tokens: recur_step_kernel does it all, a workgroup per (row, head, range of value columns).
// Portions of prompts, cut into chunks of 64 tokens, c_t = sum of the logarithms of the decays of the
// chunk's tokens up to t (every exponent below is <= 0):
//   recur_prep_*    c, dt, and the convolved inputs
//   recur_state     per chunk  U = sum_t exp(c_end - c_t) k_t v_t^T
//   recur_scores    per chunk  A[i][j] = sum_d q_i k_j exp(c_i - c_j), j <= i; decay per head: q_i . k_j
//   recur_scan      per portion, elementwise over the state: U <- state ahead of the chunk; the end state
//   recur_out       per chunk  o_i = exp(c_i) q_i S + sum_j A[i][j] v_j (+ D v_i)
// A decay per channel does not factor out of a score without overflow, so its scores are formed for
// 16-token blocks: between blocks both factors are taken to the query block's start, inside a block
// each pair has its own exponentials.
#include "../../include/exo_mi355x.h"
#include "dense.h"

namespace {

constexpr int kChunk = 64;
constexpr int kRec = 8;  // ints of a chunk's record: row, cache row, position, tokens, portion's first position

typedef exo_recurrence Rec;

__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float sigmoidf(float z) { return 1.f / (1.f + expf(-z)); }

template <typename T>
__device__ __forceinline__ const T* as(const void* p) {
  return reinterpret_cast<const T*>(p);
}

// a float32 operand of a matrix product
template <typename T>
struct Split;
template <>
struct Split<bf16_t> {
  uint4 hi, lo;
  __device__ __forceinline__ void set(const float (&f)[8]) {
    uint32_t h[4], l[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      h[i] = pack_bf2(f[2 * i], f[2 * i + 1]);
      l[i] = pack_bf2(f[2 * i] - bf_lo(h[i]), f[2 * i + 1] - bf_hi(h[i]));
    }
    hi = uint4{h[0], h[1], h[2], h[3]};
    lo = uint4{l[0], l[1], l[2], l[3]};
  }
};
template <>
struct Split<float> {
  uint4 hi;
  __device__ __forceinline__ void set(const float (&f)[4]) { hi = __builtin_bit_cast(uint4, floatx4{f[0], f[1], f[2], f[3]}); }
};
template <typename T>
__device__ __forceinline__ floatx4 mma(const Split<T>& a, const uint4& b, floatx4 c) {
  if constexpr (sizeof(T) == 2) c = Elem<T>::mma16(a.lo, b, c);
  return Elem<T>::mma16(a.hi, b, c);
}
template <typename T>
__device__ __forceinline__ floatx4 mma(const uint4& a, const Split<T>& b, floatx4 c) {
  if constexpr (sizeof(T) == 2) c = Elem<T>::mma16(a, b.lo, c);
  return Elem<T>::mma16(a, b.hi, c);
}
template <typename T>
__device__ __forceinline__ floatx4 mma(const Split<T>& a, const Split<T>& b, floatx4 c) {
  if constexpr (sizeof(T) == 2) {
    c = Elem<T>::mma16(a.lo, b.hi, c);
    c = Elem<T>::mma16(a.hi, b.lo, c);
  }
  return Elem<T>::mma16(a.hi, b.hi, c);
}

// N elements from p, zero from `left` on
template <typename T, int N>
__device__ __forceinline__ void load_n(const T* p, T (&f)[N], bool vec, int left) {
  if (vec && left >= N) {
    if constexpr (N * sizeof(T) >= 16) {
#pragma unroll
      for (int i = 0; i < (int)(N * sizeof(T) / 16); ++i)
        *reinterpret_cast<uint4*>(&f[i * 16 / sizeof(T)]) = *reinterpret_cast<const uint4*>(p + i * 16 / sizeof(T));
    } else {
      *reinterpret_cast<uint2*>(&f[0]) = *reinterpret_cast<const uint2*>(p);
    }
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) f[i] = i < left ? p[i] : T(0);
  }
}

struct Chunk {
  int row, crow, pos, n, pos0;
  __device__ __forceinline__ explicit Chunk(const int32_t* list, int i) {
    const int32_t* c = list + (size_t)i * kRec;
    row = c[0], crow = c[1], pos = c[2], n = min(c[3], kChunk), pos0 = c[4];
  }
};

// ------------------------------------------------------------------------------ what enters a recurrence
// c per key channel: z = low-rank product + bias, log decay = -softplus(-z) / tau, summed over the chunk
constexpr int kRankStep = 16, kSeg = kChunk / 4;

// 64 channels per workgroup; a wave takes a quarter of the tokens
__global__ __launch_bounds__(256) void recur_prep_channel_kernel(const Rec p) {
  __shared__ __attribute__((aligned(16))) float low[kChunk][kRankStep];
  __shared__ float total[4][64];
  const Chunk ck(p.chunks, blockIdx.x);
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane((int)threadIdx.x >> 6);
  const int c = blockIdx.y * 64 + lane, C = p.heads * p.dim, cc = min(c, C - 1), t0 = wave * kSeg;
  float acc[kSeg];
  const float b = p.decay_b[cc];
#pragma unroll
  for (int t = 0; t < kSeg; ++t) acc[t] = b;
  for (int j0 = 0; j0 < p.rank; j0 += kRankStep) {
    __syncthreads();
    for (int i = threadIdx.x; i < kChunk * kRankStep; i += 256) {
      const int t = i / kRankStep, j = i % kRankStep;
      low[t][j] = t < ck.n && j0 + j < p.rank ? p.low[(size_t)(ck.row + t) * p.ldlow + j0 + j] : 0.f;
    }
    __syncthreads();
    float w[kRankStep];
#pragma unroll
    for (int j = 0; j < kRankStep; ++j) w[j] = j0 + j < p.rank ? p.decay_w[(size_t)(j0 + j) * C + cc] : 0.f;
#pragma unroll
    for (int t = 0; t < kSeg; ++t)
#pragma unroll
      for (int j = 0; j < kRankStep; j += 4) {
        const floatx4 l = *reinterpret_cast<const floatx4*>(&low[t0 + t][j]);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[t] = fmaf(w[j + e], l[e], acc[t]);
      }
  }
  float sum = 0.f;
#pragma unroll
  for (int t = 0; t < kSeg; ++t) {
    sum -= softplus(-acc[t]) * p.inv_tau;
    acc[t] = sum;
  }
  total[wave][lane] = sum;
  __syncthreads();
  float base = 0.f;
  for (int w = 0; w < wave; ++w) base += total[w][lane];
  if (c >= C) return;
#pragma unroll
  for (int t = 0; t < kSeg; ++t)
    if (t0 + t < ck.n) p.cum[(size_t)(ck.row + t0 + t) * p.ldcum + c] = base + acc[t];
}

// c and dt per head: a wave per head, a lane per token
__global__ __launch_bounds__(256) void recur_prep_head_kernel(const Rec p) {
  const Chunk ck(p.chunks, blockIdx.x);
  const int lane = threadIdx.x & 63, h = blockIdx.y * 4 + (threadIdx.x >> 6);
  if (h >= p.heads) return;
  const bool on = lane < ck.n;
  const size_t row = (size_t)ck.row + min(lane, ck.n - 1);
  const float dt = softplus(p.dt_raw[row * p.lddt + h] + p.dt_bias[h]);
  float s = on ? -p.decay_rate[h] * dt : 0.f;
#pragma unroll
  for (int o = 1; o < 64; o *= 2) {
    const float u = __shfl_up(s, o, 64);
    if (lane >= o) s += u;
  }
  if (on) {
    p.cum[row * p.ldcum + h] = s;
    p.dt[row * p.ldcum + h] = dt;
  }
}

// causal convolution per channel and silu, 16 tokens per thread
constexpr int kConvTokens = 16;

template <typename T, int TM>
__global__ __launch_bounds__(256) void recur_conv_kernel(const Rec p) {
  const Chunk ck(p.chunks, blockIdx.x / (kChunk / kConvTokens));
  const int t0 = (blockIdx.x % (kChunk / kConvTokens)) * kConvTokens, c = blockIdx.y * 256 + threadIdx.x;
  if (t0 >= ck.n || c >= p.channels) return;
  float w[TM], x[TM];  // the latest TM inputs, oldest first (taps < TM: zero weights in front)
#pragma unroll
  for (int i = 0; i < TM; ++i) {
    const int tap = i - (TM - p.taps);
    w[i] = tap >= 0 ? p.conv_w[(size_t)tap * p.channels + c] : 0.f;
  }
  const float b = p.conv_b[c];
  const T* raw = as<T>(p.raw) + (size_t)ck.row * p.ldraw + c;
  const T* ring = as<T>(p.ring) + (size_t)p.map[ck.crow] * p.taps * p.channels + c;
#pragma unroll
  for (int i = 0; i < TM - 1; ++i) {
    const int back = TM - 1 - i, at = ck.pos + t0 - back;  // position of that input
    x[i] = 0.f;
    if (back < p.taps && at >= 0)
      x[i] = at >= ck.pos0 ? Elem<T>::load(raw[(ptrdiff_t)(t0 - back) * p.ldraw])
                           : Elem<T>::load(ring[(size_t)(at % p.taps) * p.channels]);
  }
  T in[kConvTokens];
#pragma unroll
  for (int t = 0; t < kConvTokens; ++t) in[t] = raw[(size_t)min(t0 + t, ck.n - 1) * p.ldraw];
  T* out = reinterpret_cast<T*>(p.act) + (size_t)ck.row * p.ldact + c;
#pragma unroll
  for (int t = 0; t < kConvTokens; ++t) {
    x[TM - 1] = Elem<T>::load(in[t]);
    float y = b;
#pragma unroll
    for (int i = 0; i < TM; ++i) y = fmaf(w[i], x[i], y);
    if (t0 + t < ck.n) out[(size_t)(t0 + t) * p.ldact] = Elem<T>::make(y * sigmoidf(y));
#pragma unroll
    for (int i = 0; i < TM - 1; ++i) x[i] = x[i + 1];
  }
}

// ------------------------------------------------------------------------------ chunks
// the value columns [e0, e0 + 64) of a chunk, transposed: vt[column][token], zero past n and E
template <typename T>
constexpr int kVStride = kChunk + 16 / (int)sizeof(T);

template <typename T>
__device__ __forceinline__ void stage_values(const Rec& p, const Chunk& ck, int h, int e0, T* vt, int tid) {
  const int q = (tid & 15) * 4, t0 = (tid >> 4) * 4;
  struct alignas(4 * sizeof(T)) Quad {
    T e[4];
  };
  Quad in[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = t0 + i;
    load_n<T, 4>(as<T>(p.v) + (size_t)(ck.row + min(t, ck.n - 1)) * p.ldv + h * p.vdim + e0 + q, in[i].e, p.v_vec != 0,
                 t < ck.n ? p.vdim - e0 - q : 0);
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    Quad out;
#pragma unroll
    for (int i = 0; i < 4; ++i) out.e[i] = in[i].e[e];
    *reinterpret_cast<Quad*>(vt + (q + e) * kVStride<T> + t0) = out;
  }
}

// 64 channels x 64 value columns of a chunk's own contribution to the state
template <typename T, bool CHANNEL>
__global__ __launch_bounds__(256) void recur_state_kernel(const Rec p) {
  constexpr int KV = Elem<T>::kVec;
  __shared__ __attribute__((aligned(16))) T vt[64 * kVStride<T>];
  __shared__ float wt[kChunk];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const Chunk ck(p.chunks, blockIdx.x);
  const int h = blockIdx.y, gk = h / (p.heads / p.groups);
  const int ne = (p.lds + 63) / 64, e0 = ((int)blockIdx.z % ne) * 64, d0 = ((int)blockIdx.z / ne) * 64;
  stage_values<T>(p, ck, h, e0, vt, tid);
  const size_t last = (size_t)(ck.row + ck.n - 1) * p.ldcum;
  if (!CHANNEL && tid < kChunk) {
    const size_t at = (size_t)(ck.row + min(tid, ck.n - 1)) * p.ldcum + h;
    wt[tid] = tid < ck.n ? expf(p.cum[last + h] - p.cum[at]) * p.dt[at] : 0.f;
  }
  __syncthreads();
  const int d = d0 + wave * 16 + r;
  const bool on = d < p.dim;
  const int dc = min(d, p.dim - 1);
  const float cend = CHANNEL ? p.cum[last + h * p.dim + dc] : 0.f;
  const T* kp = as<T>(p.k) + (size_t)ck.row * p.ldk + gk * p.dim + dc;
  const float* cp = p.cum + (size_t)ck.row * p.ldcum + h * p.dim + dc;
  floatx4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < kChunk; s += 4 * KV) {
    if (s >= ck.n) break;
    float f[KV];
#pragma unroll
    for (int e = 0; e < KV; ++e) {
      const int t = s + g * KV + e, tc = min(t, ck.n - 1);
      const float k = Elem<T>::load(kp[(size_t)tc * p.ldk]);
      const float w = CHANNEL ? expf(cend - cp[(size_t)tc * p.ldcum]) : wt[t];
      f[e] = on && t < ck.n ? k * w : 0.f;
    }
    Split<T> a;
    a.set(f);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      acc[j] = mma<T>(a, *reinterpret_cast<const uint4*>(vt + (j * 16 + r) * kVStride<T> + s + g * KV), acc[j]);
  }
  float* u = p.chunk_state + ((size_t)blockIdx.x * p.heads + h) * p.dim * p.lds;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int col = e0 + j * 16 + r;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int dd = d0 + wave * 16 + 4 * g + e;
      if (dd < p.dim && col < p.lds) u[(size_t)dd * p.lds + col] = acc[j][e];
    }
  }
}

// scores of a chunk, decay per head: the plain products of a group's queries and keys
template <typename T>
__global__ __launch_bounds__(256) void recur_scores_head_kernel(const Rec p) {
  constexpr int KV = Elem<T>::kVec;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane((int)threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const Chunk ck(p.chunks, blockIdx.x);
  const int grp = blockIdx.y, i0 = wave * 16;
  if (i0 >= ck.n) return;
  const T* qp = as<T>(p.q) + (size_t)(ck.row + min(i0 + r, ck.n - 1)) * p.ldq + grp * p.dim;
  const T* kp[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) kp[j] = as<T>(p.k) + (size_t)(ck.row + min(j * 16 + r, ck.n - 1)) * p.ldk + grp * p.dim;
  floatx4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = floatx4{0.f, 0.f, 0.f, 0.f};
  for (int s = 0; s < p.dim; s += 4 * KV) {
    const int d = s + g * KV, left = p.dim - d;
    struct alignas(16) Vec {
      T e[KV];
    } a, b[4];
    load_n<T, KV>(qp + d, a.e, p.qk_vec != 0, left);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wave) load_n<T, KV>(kp[j] + d, b[j].e, p.qk_vec != 0, left);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= wave) acc[j] = Elem<T>::mma16(__builtin_bit_cast(uint4, a), __builtin_bit_cast(uint4, b[j]), acc[j]);
  }
  float* out = p.scores + ((size_t)blockIdx.x * p.groups + grp) * kChunk * kChunk;
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (j <= wave) {
#pragma unroll
      for (int e = 0; e < 4; ++e) out[(i0 + 4 * g + e) * kChunk + j * 16 + r] = acc[j][e] * p.q_scale;
    }
}

// scores of a chunk, decay per key channel (queries and keys per head); 64 channels at a time in LDS
template <typename T>
__global__ __launch_bounds__(256) void recur_scores_channel_kernel(const Rec p) {
  constexpr int KV = Elem<T>::kVec, ST = 68;
  __shared__ __attribute__((aligned(16))) float qs[kChunk][ST], ks[kChunk][ST], cs[kChunk][ST];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const Chunk ck(p.chunks, blockIdx.x);
  const int h = blockIdx.y, i0 = wave * 16;
  floatx4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = floatx4{0.f, 0.f, 0.f, 0.f};
  for (int d0 = 0; d0 < p.dim; d0 += 64) {
    __syncthreads();
    {
      const int c = lane, d = d0 + c;
      const bool on = d < p.dim;
#pragma unroll 4
      for (int t = wave; t < kChunk; t += 4) {
        const bool live = on && t < ck.n;
        const size_t row = (size_t)ck.row + t;
        qs[t][c] = live ? Elem<T>::load(as<T>(p.q)[row * p.ldq + h * p.dim + d]) * p.q_scale : 0.f;
        ks[t][c] = live ? Elem<T>::load(as<T>(p.k)[row * p.ldk + h * p.dim + d]) : 0.f;
        cs[t][c] = live ? p.cum[row * p.ldcum + h * p.dim + d] : 0.f;
      }
    }
    __syncthreads();
    if (i0 >= ck.n) continue;
    const int db = min(64, p.dim - d0);
    // earlier blocks: both factors relative to the last token ahead of this wave's queries
    if (wave > 0) {
      for (int s = 0; s < db; s += 4 * KV) {
        const int d = s + g * KV;
        float base[KV], f[KV];
        Split<T> a, b;
#pragma unroll
        for (int e = 0; e < KV; ++e) {
          base[e] = cs[i0 - 1][d + e];
          f[e] = qs[i0 + r][d + e] * expf(fminf(cs[i0 + r][d + e] - base[e], 0.f));
        }
        a.set(f);
#pragma unroll
        for (int j = 0; j < 3; ++j)
          if (j < wave) {
#pragma unroll
            for (int e = 0; e < KV; ++e) f[e] = ks[j * 16 + r][d + e] * expf(base[e] - cs[j * 16 + r][d + e]);
            b.set(f);
            acc[j] = mma<T>(a, b, acc[j]);
          }
      }
    }
    // the own block, pair by pair: lane (g, r) has queries 4g .. 4g + 3 and key r
    float own[4] = {0.f, 0.f, 0.f, 0.f};
    for (int d = 0; d < db; d += 4) {
      const floatx4 k = *reinterpret_cast<const floatx4*>(&ks[i0 + r][d]), c = *reinterpret_cast<const floatx4*>(&cs[i0 + r][d]);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const floatx4 q = *reinterpret_cast<const floatx4*>(&qs[i0 + 4 * g + e][d]), b = *reinterpret_cast<const floatx4*>(&cs[i0 + 4 * g + e][d]);
#pragma unroll
        for (int i = 0; i < 4; ++i) own[e] = fmaf(q[i] * k[i], expf(fminf(b[i] - c[i], 0.f)), own[e]);
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j == wave) {
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[j][e] += own[e];
      }
  }
  if (i0 >= ck.n) return;
  float* out = p.scores + ((size_t)blockIdx.x * p.heads + h) * kChunk * kChunk;
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (j <= wave) {
#pragma unroll
      for (int e = 0; e < 4; ++e) out[(i0 + 4 * g + e) * kChunk + j * 16 + r] = acc[j][e];
    }
}

// along a portion's chunks: chunk_state becomes the state ahead of its chunk, the slot gets the last
// one.  blockIdx.y == heads: the convolution's ring takes the portion's last inputs.
template <typename T, bool CHANNEL>
__global__ __launch_bounds__(256) void recur_scan_kernel(const Rec p) {
  const int32_t* seq = p.seqs + 4 * (size_t)blockIdx.z;
  const int first = seq[0], count = seq[1];
  const Chunk c0(p.chunks, first);
  const int slot = p.map[c0.crow];
  if ((int)blockIdx.y == p.heads) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= p.channels) return;
    const Chunk cl(p.chunks, first + count - 1);
    const int end = cl.pos + cl.n;  // one past the last position
    T* ring = reinterpret_cast<T*>(p.ring) + (size_t)slot * p.taps * p.channels + c;
    for (int at = max(end - p.taps, c0.pos0); at < end; ++at)
      ring[(size_t)(at % p.taps) * p.channels] = as<T>(p.raw)[(size_t)(c0.row + at - c0.pos0) * p.ldraw + c];
    return;
  }
  const int h = blockIdx.y, i = (blockIdx.x * 256 + threadIdx.x) * 4, size = p.dim * p.lds;
  if (i >= size) return;
  const int d = i / p.lds;
  float* st = p.state + ((size_t)slot * p.heads + h) * size + i;
  floatx4 s = {0.f, 0.f, 0.f, 0.f};
  if (c0.pos0 > 0) s = *reinterpret_cast<const floatx4*>(st);
  constexpr int kAhead = 4;
  for (int b = 0; b < count; b += kAhead) {
    floatx4 u[kAhead];
    float e[kAhead];
#pragma unroll
    for (int j = 0; j < kAhead; ++j) {
      const int ci = first + min(b + j, count - 1);
      const Chunk ck(p.chunks, ci);
      u[j] = *reinterpret_cast<const floatx4*>(p.chunk_state + ((size_t)ci * p.heads + h) * size + i);
      e[j] = p.cum[(size_t)(ck.row + ck.n - 1) * p.ldcum + (CHANNEL ? h * p.dim + d : h)];
    }
#pragma unroll
    for (int j = 0; j < kAhead; ++j) {
      if (b + j >= count) break;
      *reinterpret_cast<floatx4*>(p.chunk_state + ((size_t)(first + b + j) * p.heads + h) * size + i) = s;
      const float a = expf(e[j]);
#pragma unroll
      for (int k = 0; k < 4; ++k) s[k] = fmaf(a, s[k], u[j][k]);
    }
  }
  *reinterpret_cast<floatx4*>(st) = s;
}

// 64 value columns of a chunk's outputs
template <typename T, bool CHANNEL>
__global__ __launch_bounds__(256) void recur_out_kernel(const Rec p) {
  constexpr int KV = Elem<T>::kVec, DB = 32, SS = DB + 16 / (int)sizeof(T), NT = sizeof(T) == 2 ? 2 : 1;
  __shared__ __attribute__((aligned(16))) T vt[64 * kVStride<T>];
  __shared__ __attribute__((aligned(16))) T st[NT][64 * SS];  // state columns [column][key], as (value, remainder)
  __shared__ float cl[kChunk], dl[kChunk];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const Chunk ck(p.chunks, blockIdx.x);
  const int h = blockIdx.y, grp = h / (p.heads / p.groups), e0 = (int)blockIdx.z * 64, i0 = wave * 16;
  const bool active = i0 < ck.n;
  stage_values<T>(p, ck, h, e0, vt, tid);
  if (!CHANNEL && tid < kChunk) {
    const size_t at = (size_t)(ck.row + min(tid, ck.n - 1)) * p.ldcum + h;
    cl[tid] = p.cum[at];
    dl[tid] = p.dt[at];
  }
  // ---- from the state ahead of the chunk
  floatx4 acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = floatx4{0.f, 0.f, 0.f, 0.f};
  const float* S = p.chunk_state + ((size_t)blockIdx.x * p.heads + h) * p.dim * p.lds;
  const bool start = ck.pos == 0;  // (nothing ahead of the sequence's first token)
  const int lr = ck.row + min(i0 + r, ck.n - 1);
  const T* qp = as<T>(p.q) + (size_t)lr * p.ldq + grp * p.dim;
  const float* cp = p.cum + (size_t)lr * p.ldcum + h * p.dim;
  const int q4 = (tid & 15) * 4, dp = (tid >> 4) * 2;
  floatx4 in[2];
  auto load_state = [&](int s) {
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      in[k] = floatx4{0.f, 0.f, 0.f, 0.f};
      if (s + dp + k < p.dim && e0 + q4 < p.lds) in[k] = *reinterpret_cast<const floatx4*>(S + (size_t)(s + dp + k) * p.lds + e0 + q4);
    }
  };
  if (!start) load_state(0);
  for (int s0 = 0; s0 < p.dim && !start; s0 += DB) {
    __syncthreads();  // (the previous block has been read)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int at = (q4 + e) * SS + dp;
      if constexpr (sizeof(T) == 2) {
        const uint32_t hi = pack_bf2(in[0][e], in[1][e]);
        *reinterpret_cast<uint32_t*>(&st[0][at]) = hi;
        *reinterpret_cast<uint32_t*>(&st[NT - 1][at]) = pack_bf2(in[0][e] - bf_lo(hi), in[1][e] - bf_hi(hi));
      } else {
        st[0][at] = in[0][e];
        st[0][at + 1] = in[1][e];
      }
    }
    __syncthreads();
    if (s0 + DB < p.dim) load_state(s0 + DB);
    if (!active) continue;
#pragma unroll
    for (int s = 0; s < DB; s += 4 * KV) {
      const int d = s0 + s + g * KV, left = p.dim - d;
      struct alignas(16) Vec {
        T e[KV];
      } a;
      load_n<T, KV>(qp + d, a.e, p.qk_vec != 0, left);
      Split<T> sa;
      if (CHANNEL) {
        float f[KV];
#pragma unroll
        for (int e = 0; e < KV; ++e) f[e] = e < left ? Elem<T>::load(a.e[e]) * p.q_scale * expf(cp[d + e]) : 0.f;
        sa.set(f);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        Split<T> b;
        b.hi = *reinterpret_cast<const uint4*>(&st[0][(j * 16 + r) * SS + s + g * KV]);
        if constexpr (sizeof(T) == 2) b.lo = *reinterpret_cast<const uint4*>(&st[NT - 1][(j * 16 + r) * SS + s + g * KV]);
        if (CHANNEL)
          acc[j] = mma<T>(sa, b, acc[j]);
        else
          acc[j] = mma<T>(__builtin_bit_cast(uint4, a), b, acc[j]);
      }
    }
  }
  __syncthreads();
  if (!active) return;
  if (!CHANNEL) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float f = expf(cl[i0 + 4 * g + e]) * p.q_scale;
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[j][e] *= f;
    }
  }
  // ---- from the chunk's own tokens
  const float* A = p.scores + ((size_t)blockIdx.x * p.groups + grp) * kChunk * kChunk + (i0 + r) * kChunk;
#pragma unroll
  for (int s = 0; s < kChunk; s += 4 * KV) {
    if (s > i0 + 15) break;
    float f[KV];
#pragma unroll
    for (int e4 = 0; e4 < KV; e4 += 4) {
      const int j = s + g * KV + e4;
      // (blocks of 16 keys behind the query's own are not written)
      const floatx4 v = j <= i0 + 15 ? *reinterpret_cast<const floatx4*>(A + j) : floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int jj = j + e;
        const float w = CHANNEL ? 1.f : expf(fminf(cl[i0 + r] - cl[jj], 0.f)) * dl[jj];
        f[e4 + e] = jj <= i0 + r && jj < ck.n ? v[e] * w : 0.f;
      }
    }
    Split<T> a;
    a.set(f);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      acc[j] = mma<T>(a, *reinterpret_cast<const uint4*>(vt + (j * 16 + r) * kVStride<T> + s + g * KV), acc[j]);
  }
  const float skip = p.skip ? p.skip[h] : 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int col = e0 + j * 16 + r;
    if (col >= p.vdim) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = i0 + 4 * g + e;
      if (t >= ck.n) continue;
      float y = acc[j][e];
      if (p.skip) y = fmaf(skip, Elem<T>::load(vt[(j * 16 + r) * kVStride<T> + t]), y);
      p.y[(size_t)(ck.row + t) * p.ldy + h * p.vdim + col] = y;
    }
  }
}

// ------------------------------------------------------------------------------ single tokens
// One convolved input: the current one from its row, the others from the ring; `keep`: the current one
// takes its place in the ring.
template <typename T>
__device__ __forceinline__ float conv_one(const Rec& p, int row, int slot, int pos, int c, bool keep) {
  T* ring = reinterpret_cast<T*>(p.ring) + (size_t)slot * p.taps * p.channels + c;
  const T cur = as<T>(p.raw)[(size_t)row * p.ldraw + c];
  float y = p.conv_b[c];
  for (int i = 0; i < p.taps - 1; ++i) {
    const int at = pos - (p.taps - 1) + i;
    if (at >= 0) y = fmaf(p.conv_w[(size_t)i * p.channels + c], Elem<T>::load(ring[(size_t)(at % p.taps) * p.channels]), y);
  }
  y = fmaf(p.conv_w[(size_t)(p.taps - 1) * p.channels + c], Elem<T>::load(cur), y);
  if (keep) ring[(size_t)(pos % p.taps) * p.channels] = cur;
  return Elem<T>::load(Elem<T>::make(y * sigmoidf(y)));
}

template <typename T, bool CHANNEL>
__global__ __launch_bounds__(256) void recur_step_kernel(const Rec p, int cols) {
  extern __shared__ __attribute__((aligned(16))) float lds[];  // q, k, decay [dim]; values [64]; partials [1024]
  const int tid = threadIdx.x, D = p.dim, h = blockIdx.y, e0 = blockIdx.x * cols;
  const int Dp = (D + 3) / 4 * 4;
  float *qs = lds, *ks = qs + Dp, *as_ = ks + Dp, *vs = as_ + Dp, *red = vs + 64;
  const int row = p.list ? p.list[blockIdx.z] : (int)blockIdx.z;
  const int crow = p.slot[row], pos = p.pos[row], slot = p.map[crow];
  const int hpg = p.heads / p.groups, grp = h / hpg;
  // this thread's part of the state is requested ahead of everything it depends on
  const int lpr = cols / 4, cq = (tid % lpr) * 4, dr = tid / lpr, rpp = 256 / lpr;
  const bool on = e0 + cq < p.lds;
  float* st = p.state + ((size_t)slot * p.heads + h) * D * p.lds + e0 + cq;
  constexpr int kAhead = 8;
  floatx4 s[kAhead];
  auto load_state = [&](int d0) {
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      s[i] = floatx4{0.f, 0.f, 0.f, 0.f};
      const int d = d0 + i * rpp;
      if (on && pos > 0 && d < D) s[i] = *reinterpret_cast<const floatx4*>(st + (size_t)d * p.lds);
    }
  };
  load_state(dr);
  float vscale = 1.f, skip = 0.f;
  if (CHANNEL) {
    const int C = p.heads * D;
    const float* low = p.low + (size_t)row * p.ldlow;
    for (int d = tid; d < D; d += 256) {
      const int c = h * D + d;
      float z = p.decay_b[c];
      for (int j = 0; j < p.rank; ++j) z = fmaf(p.decay_w[(size_t)j * C + c], low[j], z);
      as_[d] = expf(-softplus(-z) * p.inv_tau);
      qs[d] = Elem<T>::load(as<T>(p.q)[(size_t)row * p.ldq + grp * D + d]) * p.q_scale;
      ks[d] = Elem<T>::load(as<T>(p.k)[(size_t)row * p.ldk + grp * D + d]);
    }
    if (tid < cols) vs[tid] = e0 + tid < p.vdim ? Elem<T>::load(as<T>(p.v)[(size_t)row * p.ldv + h * p.vdim + e0 + tid]) : 0.f;
  } else {
    const bool keep = blockIdx.x == 0 && h == grp * hpg;  // a group's keys and queries: one workgroup's to keep
    for (int d = tid; d < D; d += 256) {
      ks[d] = conv_one<T>(p, row, slot, pos, p.k_channel + grp * D + d, keep);
      qs[d] = conv_one<T>(p, row, slot, pos, p.q_channel + grp * D + d, keep) * p.q_scale;
    }
    if (tid >= 192 && tid - 192 < cols) {
      const int e = e0 + tid - 192;
      vs[tid - 192] = e < p.vdim ? conv_one<T>(p, row, slot, pos, p.v_channel + h * p.vdim + e, true) : 0.f;
    }
    vscale = softplus(p.dt_raw[(size_t)row * p.lddt + h] + p.dt_bias[h]);
    const float a = expf(-p.decay_rate[h] * vscale);
    for (int d = tid; d < D; d += 256) as_[d] = a;
    if (p.skip) skip = p.skip[h];
  }
  __syncthreads();
  floatx4 v, o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = vs[cq + e] * vscale;
  for (int d0 = dr; d0 < D; d0 += kAhead * rpp) {
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int d = d0 + i * rpp;
      if (d >= D) break;
      const float a = as_[d], k = ks[d], q = qs[d];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        s[i][e] = fmaf(a, s[i][e], k * v[e]);
        o[e] = fmaf(q, s[i][e], o[e]);
      }
      if (on) *reinterpret_cast<floatx4*>(st + (size_t)d * p.lds) = s[i];
    }
    if (d0 + kAhead * rpp < D) load_state(d0 + kAhead * rpp);
  }
  *reinterpret_cast<floatx4*>(red + dr * cols + cq) = o;
  __syncthreads();
  if (tid < cols && e0 + tid < p.vdim) {
    float y = 0.f;
    for (int i = 0; i < rpp; ++i) y += red[i * cols + tid];
    p.y[(size_t)row * p.ldy + h * p.vdim + e0 + tid] = fmaf(skip, vs[tid], y);
  }
}

// ------------------------------------------------------------------------------ gated norm
// out = norm of equal parts of y, with the gate silu(z) ahead of the norm or behind it; the gain
// repeats with `period`.  A team of TEAM threads per part.
template <typename T, int TEAM>
__global__ __launch_bounds__(256) void gated_norm_kernel(const exo_gated_norm p, const int32_t* __restrict__ rows) {
  __shared__ float part[4];
  const int tid = threadIdx.x, team = tid / TEAM, l = tid % TEAM;
  const int gi = blockIdx.x * (256 / TEAM) + team;
  const int row = rows ? rows[blockIdx.y] : (int)blockIdx.y;
  const int size = p.width / p.groups;
  const bool on = gi < p.groups;
  const float* y = p.y + (size_t)row * p.ldy + (size_t)gi * size;
  const T* z = as<T>(p.gate) + (size_t)row * p.ldg + (size_t)gi * size;
  float ss = 0.f;
  if (on)
    for (int c = l; c < size; c += TEAM) {
      float v = y[c];
      if (p.gate_first) {
        const float zz = Elem<T>::load(z[c]);
        v *= zz * sigmoidf(zz);
      }
      ss += v * v;
    }
  ss = wave_sum(ss);
  if (TEAM == 256) {
    if ((tid & 63) == 0) part[tid >> 6] = ss;
    __syncthreads();
    ss = part[0] + part[1] + part[2] + part[3];
  }
  if (!on) return;
  const float inv = 1.f / sqrtf(ss / size + p.eps);
  T* out = reinterpret_cast<T*>(p.out) + (size_t)row * p.ldo + (size_t)gi * size;
  for (int c = l; c < size; c += TEAM) {
    const float zz = Elem<T>::load(z[c]), gate = zz * sigmoidf(zz);
    const float v = p.gate_first ? y[c] * gate : y[c];
    const float w = p.gain[(gi * size + c) % p.period];
    out[c] = Elem<T>::make(p.gate_first ? v * inv * w : v * inv * w * gate);
  }
}

int check(const Rec* a, const char* what) {
  EXO_REQUIRE(a && (a->dtype == 0 || a->dtype == 1), "%s: bad dtype", what);
  EXO_REQUIRE(a->heads > 0 && a->groups > 0 && a->heads % a->groups == 0 && a->dim > 0 && a->dim <= 1024 && a->vdim > 0 &&
                  a->lds >= a->vdim && a->lds % 4 == 0,
              "%s: bad sizes (heads=%d groups=%d dim=%d vdim=%d stride=%d)", what, a->heads, a->groups, a->dim, a->vdim, a->lds);
  EXO_REQUIRE(a->heads <= 65534, "%s: %d heads", what, a->heads);
  EXO_REQUIRE(a->state && a->map && a->y && a->ldy >= a->heads * a->vdim && ((uintptr_t)a->state & 15) == 0, "%s: bad state or output", what);
  if (a->per_channel) {
    EXO_REQUIRE(a->groups == a->heads && a->taps == 0 && !a->skip, "%s: a decay per channel goes with queries and keys per head, no convolution", what);
    EXO_REQUIRE(a->low && a->decay_w && a->decay_b && a->rank > 0 && a->ldlow >= a->rank, "%s: incomplete decay", what);
  } else {
    EXO_REQUIRE(a->dt_raw && a->dt_bias && a->decay_rate && a->lddt >= a->heads, "%s: incomplete step sizes", what);
    EXO_REQUIRE(a->taps > 0 && a->taps <= 16 && a->raw && a->ring && a->conv_w && a->conv_b && a->ldraw >= a->channels,
                "%s: incomplete convolution (%d taps, at most 16)", what, a->taps);
    EXO_REQUIRE(a->v_channel >= 0 && a->v_channel + a->heads * a->vdim <= a->channels && a->k_channel >= 0 &&
                    a->k_channel + a->groups * a->dim <= a->channels && a->q_channel >= 0 &&
                    a->q_channel + a->groups * a->dim <= a->channels,
                "%s: values, keys and queries do not lie inside the %d channels", what, a->channels);
  }
  return EXO_OK;
}

template <typename T>
bool vec_ok(const void* p, int ld, int part, int n) {
  return part % n == 0 && ld % n == 0 && (uintptr_t)p % (n * sizeof(T)) == 0;
}

template <typename T, bool CHANNEL>
void launch_chunks(Rec p, hipStream_t st) {
  constexpr int KV = Elem<T>::kVec;
  p.qk_vec = vec_ok<T>(p.q, p.ldq, p.dim, KV) && vec_ok<T>(p.k, p.ldk, p.dim, KV);
  p.v_vec = vec_ok<T>(p.v, p.ldv, p.vdim, 4);
  if constexpr (CHANNEL) {
    recur_prep_channel_kernel<<<dim3(p.n_chunks, exo_ceil_div(p.heads * p.dim, 64)), 256, 0, st>>>(p);
  } else {
    recur_prep_head_kernel<<<dim3(p.n_chunks, exo_ceil_div(p.heads, 4)), 256, 0, st>>>(p);
    const dim3 grid(p.n_chunks * (kChunk / kConvTokens), exo_ceil_div(p.channels, 256));
    if (p.taps <= 4)
      recur_conv_kernel<T, 4><<<grid, 256, 0, st>>>(p);
    else if (p.taps <= 8)
      recur_conv_kernel<T, 8><<<grid, 256, 0, st>>>(p);
    else
      recur_conv_kernel<T, 16><<<grid, 256, 0, st>>>(p);
  }
  const int ne = exo_ceil_div(p.lds, 64);
  recur_state_kernel<T, CHANNEL><<<dim3(p.n_chunks, p.heads, ne * exo_ceil_div(p.dim, 64)), 256, 0, st>>>(p);
  if constexpr (CHANNEL)
    recur_scores_channel_kernel<T><<<dim3(p.n_chunks, p.heads), 256, 0, st>>>(p);
  else
    recur_scores_head_kernel<T><<<dim3(p.n_chunks, p.groups), 256, 0, st>>>(p);
  int gx = exo_ceil_div((int64_t)p.dim * p.lds, 1024);
  if (p.taps > 0 && gx < exo_ceil_div(p.channels, 256)) gx = exo_ceil_div(p.channels, 256);
  recur_scan_kernel<T, CHANNEL><<<dim3(gx, p.heads + (p.taps > 0 ? 1 : 0), p.n_seqs), 256, 0, st>>>(p);
  recur_out_kernel<T, CHANNEL><<<dim3(p.n_chunks, p.heads, exo_ceil_div(p.vdim, 64)), 256, 0, st>>>(p);
}

template <typename T, bool CHANNEL>
void launch_step(const Rec& p, hipStream_t st) {
  int cols = 64;
  while (cols > 16 && (int64_t)p.n * p.heads * exo_ceil_div(p.lds, cols) < 256) cols /= 2;
  const int lds = (3 * ((p.dim + 3) / 4 * 4) + 64 + 1024) * 4;
  recur_step_kernel<T, CHANNEL><<<dim3(exo_ceil_div(p.lds, cols), p.heads, p.n), 256, lds, st>>>(p, cols);
}

}  // namespace

extern "C" int64_t exo_recur_scores_floats(int n_chunks, int groups) { return (int64_t)n_chunks * groups * kChunk * kChunk; }
extern "C" int64_t exo_recur_state_floats(int n_chunks, int heads, int dim, int lds) {
  return (int64_t)n_chunks * heads * dim * lds;
}
extern "C" int exo_recur_chunk(void) { return kChunk; }

extern "C" int exo_recur_chunks(const exo_recurrence* a, exo_stream_t stream) {
  const int rc = check(a, "exo_recur_chunks");
  if (rc) return rc;
  EXO_REQUIRE(a->n_chunks > 0 && a->n_chunks <= 65535 && a->n_seqs > 0 && a->n_seqs <= 65535 && a->chunks && a->seqs,
              "exo_recur_chunks: bad lists (%d chunks, %d portions)", a->n_chunks, a->n_seqs);
  EXO_REQUIRE(a->q && a->k && a->v && a->cum && a->scores && a->chunk_state &&
                  a->ldcum >= (a->per_channel ? a->heads * a->dim : a->heads) && a->ldq >= a->groups * a->dim &&
                  a->ldk >= a->groups * a->dim && a->ldv >= a->heads * a->vdim && (((uintptr_t)a->scores | (uintptr_t)a->chunk_state) & 15) == 0,
              "exo_recur_chunks: bad inputs or workspace");
  EXO_REQUIRE(a->per_channel || (a->act && a->dt && a->ldact >= a->channels), "exo_recur_chunks: no place for the convolved inputs");
  if (a->dtype == 0)
    a->per_channel ? launch_chunks<bf16_t, true>(*a, (hipStream_t)stream) : launch_chunks<bf16_t, false>(*a, (hipStream_t)stream);
  else
    a->per_channel ? launch_chunks<float, true>(*a, (hipStream_t)stream) : launch_chunks<float, false>(*a, (hipStream_t)stream);
  EXO_CHECK_LAUNCH("exo_recur_chunks");
  return EXO_OK;
}

extern "C" int exo_recur_step(const exo_recurrence* a, exo_stream_t stream) {
  const int rc = check(a, "exo_recur_step");
  if (rc) return rc;
  EXO_REQUIRE(a->n > 0 && a->n <= 65535 && a->slot && a->pos, "exo_recur_step: bad rows (n=%d)", a->n);
  EXO_REQUIRE(!a->per_channel || (a->q && a->k && a->v && a->ldq >= a->heads * a->dim && a->ldk >= a->heads * a->dim && a->ldv >= a->heads * a->vdim),
              "exo_recur_step: bad inputs");
  if (a->dtype == 0)
    a->per_channel ? launch_step<bf16_t, true>(*a, (hipStream_t)stream) : launch_step<bf16_t, false>(*a, (hipStream_t)stream);
  else
    a->per_channel ? launch_step<float, true>(*a, (hipStream_t)stream) : launch_step<float, false>(*a, (hipStream_t)stream);
  EXO_CHECK_LAUNCH("exo_recur_step");
  return EXO_OK;
}

extern "C" int exo_gated_norm_rows(const exo_gated_norm* a, const int32_t* rows, int n, exo_stream_t stream) {
  EXO_REQUIRE(a && (a->dtype == 0 || a->dtype == 1) && a->y && a->gate && a->gain && a->out && n >= 0 && n <= 65535,
              "exo_gated_norm_rows: bad argument");
  EXO_REQUIRE(a->width > 0 && a->groups > 0 && a->width % a->groups == 0 && a->period > 0 && a->width % a->period == 0 &&
                  a->ldy >= a->width && a->ldg >= a->width && a->ldo >= a->width,
              "exo_gated_norm_rows: bad sizes (width=%d groups=%d period=%d)", a->width, a->groups, a->period);
  if (n == 0) return EXO_OK;
  const bool wide = a->width / a->groups > 512;
  const dim3 grid(wide ? a->groups : exo_ceil_div(a->groups, 4), n);
  const hipStream_t st = (hipStream_t)stream;
  if (a->dtype == 0)
    wide ? gated_norm_kernel<bf16_t, 256><<<grid, 256, 0, st>>>(*a, rows) : gated_norm_kernel<bf16_t, 64><<<grid, 256, 0, st>>>(*a, rows);
  else
    wide ? gated_norm_kernel<float, 256><<<grid, 256, 0, st>>>(*a, rows) : gated_norm_kernel<float, 64><<<grid, 256, 0, st>>>(*a, rows);
  EXO_CHECK_LAUNCH("exo_gated_norm_rows");
  return EXO_OK;
}
