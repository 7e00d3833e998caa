// Latent attention: a position's keys and values are linear images of one normed latent vector c, and a
// rotated key part is shared by all heads.  The paged pool holds c and that part alone:
//   pool  [page][64][ldk]   c at 0, the rotated part at c32 (the latent size rounded up to 32), zeros between
//                           and behind
// Two ways over it:
//   absorbed   (single tokens, short portions, the 32-bit mode)  A head's query goes through its key
//              matrix once, q' = W_uk^T q, and then scores the latents themselves; the weighted sum of
//              latents goes through the head's value matrix.  All heads read the same keys, so the up to
//              16 heads of a workgroup are the columns of 16x16 products, as queries of one kv head are in
//              paged_attn.hip.  exo_head_linear is the product with a matrix per head on either side.
//   expanded   (portions of prompts)  The visible latents are gathered into rows, two matrix products
//              give every head's keys (a position a row) and values (a column a row, positions in a run),
//              and the prompt kernel of paged_attn.hip reads those.
//
// latent_rows_kernel: one query position and up to 16 heads per workgroup.  A tile of keys (64, or 32 in
// the 32-bit mode) is staged in LDS once and read twice: as rows for the scores, and transposed on the way
// out of LDS for the weighted sum - four of the eight waves score 16 keys
// each, then each wave sums an eighth of the latent's columns over all of them.  The next tile is in registers meanwhile.  Splits leave float32 partials that the
// following product with the value matrices merges while it stages its operand.
#include "../../include/exo_mi355x.h"
#include "dense.h"
#include "rotary.h"
#include "route.h"

namespace {

constexpr int kPage = 64;
constexpr int kWaves = 4;
constexpr int kRowWaves = 8, kRowThreads = 64 * kRowWaves;  // of latent_rows_kernel
constexpr int kMaxRot = 128;
constexpr float kLog2e = 1.4426950408889634f;
constexpr int kPRow = 144;  // bytes of a head's weights of one tile in LDS

struct Params {
  const void* q;        // T [R][ldq]: rotated parts of head h at rot_col + h * r8
  const void* ql;       // T [R][ldql]: absorbed query of head h at h * cp
  const float* kv;      // [R][ldkv]: latent (not normed), rotated part (not turned)
  const float* gain;    // [C]
  const double* freq;   // [rot / 2] turns per position
  void* pool;
  const int32_t *table, *slot, *pos, *list;
  void* out;            // T [R][ldo]: weighted latents of head h at h * cp
  float* parts;         // [n][H][nsplit][c32 + 4]
  float scale, eps;
  int n, H, C, rot, c32, r8, cp, rot_col, ldq, ldql, ldkv, ldk, ldo, max_pages, prepared, nsplit, gsz;
};

Params params_of(const exo_latent_attn* a) {
  Params p{};
  p.q = a->q, p.ql = a->q_latent, p.kv = a->kv, p.gain = a->gain, p.freq = a->freq, p.pool = a->pool;
  p.table = a->table, p.slot = a->slot, p.pos = a->pos, p.list = a->list, p.out = a->out, p.parts = a->parts;
  p.scale = a->scale, p.eps = a->eps, p.n = a->n, p.H = a->heads, p.C = a->rank, p.rot = a->rot;
  p.c32 = (a->rank + 31) / 32 * 32, p.r8 = (a->rot + 7) / 8 * 8, p.cp = (a->rank + 63) / 64 * 64;
  p.rot_col = a->rot_col, p.ldq = a->ldq, p.ldql = a->ldql, p.ldkv = a->ldkv, p.ldk = a->ldk, p.ldo = a->ldo;
  p.max_pages = a->max_pages, p.prepared = a->prepared, p.nsplit = a->nsplit;
  return p;
}

// one wave: the row's latent, normed, into its place in the pool
template <typename T>
__device__ __forceinline__ void put_latent(const Params& p, int row, T* dst, int lane) {
  const float* src = p.kv + (size_t)row * p.ldkv;
  float v[8], ss = 0.f;  // C <= 512
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    v[i] = lane + 64 * i < p.C ? src[lane + 64 * i] : 0.f;
    ss += v[i] * v[i];
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / p.C + p.eps);
#pragma unroll
  for (int i = 0; i < 8; ++i)
    if (lane + 64 * i < p.C) dst[lane + 64 * i] = Elem<T>::make(v[i] * inv * p.gain[lane + 64 * i]);
}
// ... and the shared key part, turned
template <typename T>
__device__ __forceinline__ void put_rotated(const Params& p, int row, T* dst, const float2* cs, int lane) {
  const float* src = p.kv + (size_t)row * p.ldkv + p.C;
  for (int i = lane; 2 * i < p.rot; i += 64) {
    const float2 x = turn_pair(src[2 * i], src[2 * i + 1], cs[i]);
    dst[p.c32 + 2 * i] = Elem<T>::make(x.x), dst[p.c32 + 2 * i + 1] = Elem<T>::make(x.y);
  }
}
template <typename T>
__device__ __forceinline__ T* pool_row(const Params& p, int page, int at) {
  return reinterpret_cast<T*>(p.pool) + ((size_t)page * kPage + at) * p.ldk;
}

// ------------------------------------------------------------------------------ all rows of a step
// a wave per row: latent and shared key part into the pool, the queries' rotated parts turned in place
template <typename T>
__global__ __launch_bounds__(64 * kWaves) void latent_prepare_kernel(const Params p) {
  __shared__ float2 cs_all[kWaves][kMaxRot / 2];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane((int)threadIdx.x >> 6);
  const int row = blockIdx.x * kWaves + wave;
  if (row >= p.n) return;
  float2* cs = cs_all[wave];  // (written and read by this wave only)
  const int pos = p.pos[row];
  T* dst = pool_row<T>(p, p.table[(size_t)p.slot[row] * p.max_pages + pos / kPage], pos % kPage);
  for (int i = lane; 2 * i < p.rot; i += 64) cs[i] = turn_of(pos, p.freq[i]);
  put_latent<T>(p, row, dst, lane);
  put_rotated<T>(p, row, dst, cs, lane);
  T* q = const_cast<T*>(reinterpret_cast<const T*>(p.q)) + (size_t)row * p.ldq + p.rot_col;
  const int half = p.rot / 2;
  for (int i = lane; i < p.H * half; i += 64) {
    const int h = i / half, d = i - h * half;
    T* at = q + h * p.r8 + 2 * d;
    const float2 x = turn_pair(Elem<T>::load(at[0]), Elem<T>::load(at[1]), cs[d]);
    at[0] = Elem<T>::make(x.x), at[1] = Elem<T>::make(x.y);
  }
}

// ------------------------------------------------------------------------------ absorbed
// A lane's share of 32 (bf16) or 16 (float) keys of 16 columns, transposed out of the key tile in LDS:
// the A operand "columns x keys".  bf16: each run of 16 lanes reads four rows of 16 columns per
// instruction and receives them transposed.
template <typename T>
__device__ __forceinline__ uint4 transposed(const char* tile, int stride, int key0, int col0, int r, int g);
template <>
__device__ __forceinline__ uint4 transposed<bf16_t>(const char* tile, int stride, int key0, int col0, int r, int g) {
  typedef __attribute__((__vector_size__(4 * sizeof(short)))) short short4_t;
  typedef __attribute__((address_space(3))) short4_t* lds_ptr;
  const char* at = tile + (key0 + 8 * g + (r >> 2)) * stride + (col0 + 4 * (r & 3)) * 2;
  const short4_t a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)at);
  const short4_t b = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_ptr)(at + 4 * stride));
  const uint2 x = __builtin_bit_cast(uint2, a), y = __builtin_bit_cast(uint2, b);
  return uint4{x.x, x.y, y.x, y.y};
}
template <>
__device__ __forceinline__ uint4 transposed<float>(const char* tile, int stride, int key0, int col0, int r, int g) {
  floatx4 v;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = *reinterpret_cast<const float*>(tile + (key0 + 4 * g + i) * stride + (col0 + r) * 4);
  return __builtin_bit_cast(uint4, v);
}

template <typename T, int KMAX, bool FUSE>
__global__ __launch_bounds__(kRowThreads) void latent_rows_kernel(const Params p) {
  constexpr int ES = (int)sizeof(T), KT = ES == 2 ? 64 : 32;     // keys per tile
  constexpr int KS = KMAX * ES / 64;                             // 64-byte steps over a key
  constexpr int LOADS = (KT * KMAX * ES / 16 + kRowThreads - 1) / kRowThreads;
  constexpr int OT = ((KMAX < 512 ? KMAX : 512) / 16 + kRowWaves - 1) / kRowWaves;  // 16-column tiles of the sum per wave
  constexpr int PK = 64 / ES;                                    // keys per product of the second kind
  extern __shared__ __attribute__((aligned(16))) char lds[];
  constexpr int SW = KT / 16;                                    // waves that score
  __shared__ float wm[SW][16], wl[SW][16];
  __shared__ float2 cs[kMaxRot / 2];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int split = blockIdx.x, h0 = blockIdx.y * p.gsz, gs = min(p.gsz, p.H - h0);
  const int row = p.list ? p.list[blockIdx.z] : (int)blockIdx.z;
  const int pos = p.pos[row], nt = pos / KT + 1;
  const int32_t* table = p.table + (size_t)p.slot[row] * p.max_pages;
  const int stride = p.ldk * ES + 16, vpr = p.ldk * ES / 16, nvec = KT * vpr;
  const int ksteps = p.ldk * ES / 64, dtiles = p.c32 / 16;
  char* pw = lds + KT * stride;  // weights of the tile: [16][kPRow], bf16: high terms, then remainders

  // a tile is one run of memory; row of vector v by a reciprocal (v * vpr < 2^20: exact)
  const uint32_t magic = ((1u << 20) + vpr - 1) / vpr;
  uint4 reg[LOADS];
  auto load_tile = [&](int j) __attribute__((always_inline)) {
    const int key0 = j * KT;
    const char* src = reinterpret_cast<const char*>(pool_row<T>(p, table[key0 / kPage], key0 % kPage));
#pragma unroll
    for (int i = 0; i < LOADS; ++i)
      reg[i] = load16(src + (size_t)min(tid + kRowThreads * i, nvec - 1) * 16);
  };
  int j = split;
  const bool early = j < nt && !(FUSE && j == nt - 1);  // (not the tile that the row's own key goes into)
  if (early) load_tile(j);

  // ---- queries: absorbed part, turned part, zeros; the row's own latent
  for (int i = tid; 2 * i < p.rot; i += kRowThreads) cs[i] = turn_of(pos, p.freq[i]);
  const int cvec = p.c32 * ES / 16;
  for (int i = tid; i < 16 * vpr; i += kRowThreads) {
    const int h = (i * magic) >> 20, c = i - h * vpr;
    uint4 v{0, 0, 0, 0};
    if (h < gs && c < cvec)
      v = *reinterpret_cast<const uint4*>(reinterpret_cast<const T*>(p.ql) + (size_t)row * p.ldql + (size_t)(h0 + h) * p.cp + c * (16 / ES));
    *reinterpret_cast<uint4*>(lds + h * stride + c * 16) = v;
  }
  __syncthreads();
  const int half = p.rot / 2;
  for (int i = tid; i < gs * half; i += kRowThreads) {
    const int h = i / half, d = i - h * half;
    const T* src = reinterpret_cast<const T*>(p.q) + (size_t)row * p.ldq + p.rot_col + (h0 + h) * p.r8 + 2 * d;
    float2 x{Elem<T>::load(src[0]), Elem<T>::load(src[1])};
    if (!p.prepared) x = turn_pair(x.x, x.y, cs[d]);
    T* dst = reinterpret_cast<T*>(lds + h * stride) + p.c32 + 2 * d;
    dst[0] = Elem<T>::make(x.x), dst[1] = Elem<T>::make(x.y);
  }
  if (FUSE && split == (nt - 1) % p.nsplit) {
    T* dst = pool_row<T>(p, table[pos / kPage], pos % kPage);
    if (wave == kRowWaves - 1) put_latent<T>(p, row, dst, lane);
    if (wave == kRowWaves - 2) put_rotated<T>(p, row, dst, cs, lane);
    wait_own_stores_done();
  }
  __syncthreads();
  if (!early && j < nt) load_tile(j);
  uint4 q[KS];
#pragma unroll
  for (int s = 0; s < KS; ++s) {  // (steps past the key: zeros times its last step again, no branch in the loops)
    q[s] = load16(lds + r * stride + min(s, ksteps - 1) * 64 + g * 16);
    if (s >= ksteps) q[s] = uint4{0, 0, 0, 0};
  }
  __syncthreads();

  const float sc = p.scale * kLog2e;
  floatx4 o[OT];
#pragma unroll
  for (int t = 0; t < OT; ++t) o[t] = floatx4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  for (; j < nt; j += p.nsplit) {
#pragma unroll
    for (int i = 0; i < LOADS; ++i) {
      const uint32_t v = tid + kRowThreads * i;
      if ((int)v < nvec) *reinterpret_cast<uint4*>(lds + v * 16 + ((v * magic) >> 20) * 16) = reg[i];
    }
    if (j + p.nsplit < nt) load_tile(j + p.nsplit);
    __syncthreads();
    float x[4], mx = -INFINITY;
    if (wave < SW) {
      floatx4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
      const char* kr = lds + (wave * 16 + r) * stride + g * 16;
#pragma unroll
      for (int s = 0; s < KS; s += 2) {
        s0 = Elem<T>::mma16(load16(kr + min(s, ksteps - 1) * 64), q[s], s0);
        if (s + 1 < KS) s1 = Elem<T>::mma16(load16(kr + min(s + 1, ksteps - 1) * 64), q[s + 1 < KS ? s + 1 : s], s1);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        x[e] = j * KT + wave * 16 + 4 * g + e <= pos ? (s0[e] + s1[e]) * sc : -INFINITY;
        mx = fmaxf(mx, x[e]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    }
    if (wave < SW && g == 0) wm[wave][r] = mx;
    __syncthreads();
    float mn = m;
#pragma unroll
    for (int w = 0; w < SW; ++w) mn = fmaxf(mn, wm[w][r]);  // finite: a dealt tile holds a visible key
    const float a = __builtin_amdgcn_exp2f(m - mn);
    m = mn;
    float sum = 0.f;
    if (wave < SW) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        x[e] = __builtin_amdgcn_exp2f(x[e] - mn);
        sum += x[e];
      }
      sum += __shfl_xor(sum, 16, 64);
      sum += __shfl_xor(sum, 32, 64);
      char* dst = pw + r * kPRow + (wave * 16 + 4 * g) * ES;
      if (ES == 2) {
        float b[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) b[e] = x[e] - bf2f(f2bf(x[e]));
        *reinterpret_cast<uint2*>(dst) = uint2{pack_bf2(x[0], x[1]), pack_bf2(x[2], x[3])};
        *reinterpret_cast<uint2*>(dst + 16 * kPRow) = uint2{pack_bf2(b[0], b[1]), pack_bf2(b[2], b[3])};
      } else {
        *reinterpret_cast<floatx4*>(dst) = floatx4{x[0], x[1], x[2], x[3]};
      }
    }
    if (wave < SW && g == 0) wl[wave][r] = sum;
    __syncthreads();
    l *= a;
#pragma unroll
    for (int w = 0; w < SW; ++w) l += wl[w][r];
#pragma unroll
    for (int t = 0; t < OT; ++t)
#pragma unroll
      for (int e = 0; e < 4; ++e) o[t][e] *= a;
#pragma unroll
    for (int k = 0; k < KT / PK; ++k) {
      const uint4 hi = *reinterpret_cast<const uint4*>(pw + r * kPRow + k * 64 + g * 16);
      const uint4 lo = ES == 2 ? *reinterpret_cast<const uint4*>(pw + (16 + r) * kPRow + k * 64 + g * 16) : hi;
#pragma unroll
      for (int t = 0; t < OT; ++t) {
        const uint4 v = transposed<T>(lds, stride, k * PK, min(wave + kRowWaves * t, dtiles - 1) * 16, r, g);
        o[t] = Elem<T>::mma16(v, hi, o[t]);
        if (ES == 2) o[t] = Elem<T>::mma16(v, lo, o[t]);
      }
    }
    __syncthreads();  // the tile and its weights are no longer read
  }
  if (r >= gs) return;
  if (p.nsplit == 1) {
    const float inv = 1.f / l;
    T* out = reinterpret_cast<T*>(p.out) + (size_t)row * p.ldo + (size_t)(h0 + r) * p.cp;
#pragma unroll
    for (int t = 0; t < OT; ++t) {
      const int d = (wave + kRowWaves * t) * 16 + 4 * g;
      if (d < p.c32) {
#pragma unroll
        for (int e = 0; e < 4; ++e) out[d + e] = Elem<T>::make(o[t][e] * inv);
      }
    }
    return;
  }
  float* part = p.parts + (((size_t)blockIdx.z * p.H + h0 + r) * p.nsplit + split) * (p.c32 + 4);
#pragma unroll
  for (int t = 0; t < OT; ++t) {
    const int d = (wave + kRowWaves * t) * 16 + 4 * g;
    if (d < p.c32) *reinterpret_cast<floatx4*>(part + d) = o[t];
  }
  if (wave == 0 && g == 0) part[p.c32] = m, part[p.c32 + 1] = l;
}

// ------------------------------------------------------------------------------ a matrix per head
// y[row][h] = w[h] x[row][h]: outputs of one head and up to 16 rows per workgroup, 16x16 tiles, a wave per
// tile.  With partials of split attention x is formed from them on the way into LDS, with few rows in several
// groups of splits side by side (what counts then is how many loads follow each other), and a tile's product
// is dealt out over four waves.
struct HeadLinear {
  const void* x;        // T [R][ldx], head h at h * xh
  const float* parts;   // [n][H][nsplit][K32 + 4], or null
  const void* w;        // T [H][N][ldw]
  void* y;              // T [R][ldy], head h at h * yh
  const int32_t* list;
  int n, H, N, K32, ldx, xh, ldw, ldy, yh, nsplit;
};
constexpr int kHeadBatch = 8;
constexpr int kMaxSplits = 64;

template <typename T, bool PARTS>
__global__ __launch_bounds__(PARTS ? 512 : 256) void head_linear_kernel(const HeadLinear p) {
  constexpr int KW = PARTS ? 4 : 1, NW = PARTS ? 8 : 4, TH = 64 * NW;
  __shared__ floatx4 red[KW == 1 ? 1 : NW][KW == 1 ? 1 : 64];
  extern __shared__ __attribute__((aligned(16))) char xs[];  // PARTS: [rows][ldw * sizeof(T) + 16]
  __shared__ floatx4 sums[PARTS ? TH : 1];
  __shared__ float fac[PARTS ? 16 : 1][PARTS ? kMaxSplits : 1];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 15, g = lane >> 4, h = blockIdx.y;
  const int i0 = blockIdx.z * 16, rows = min(16, p.n - i0);
  const int n0 = (blockIdx.x * (NW / KW) + wave / KW) * 16;
  const int ri = i0 + min(r, rows - 1), row = p.list ? p.list[ri] : ri;
  const int all = p.ldw * (int)sizeof(T) / 64, each = (all + KW - 1) / KW;
  const int first = min(wave % KW * each, all), steps = min(all, first + each), lrow = p.ldw * (int)sizeof(T) + 16;
  const char* wp = reinterpret_cast<const char*>(reinterpret_cast<const T*>(p.w) + ((size_t)h * p.N + min(n0 + r, p.N - 1)) * p.ldw) + g * 16;
  const char* xp = reinterpret_cast<const char*>(reinterpret_cast<const T*>(p.x) + (size_t)row * p.ldx + (size_t)h * p.xh) + g * 16;
  uint4 wv[kHeadBatch];
  auto load_w = [&](int s) {
#pragma unroll
    for (int i = 0; i < kHeadBatch; ++i) wv[i] = load16(wp + min(s + i, all - 1) * 64);
  };
  load_w(first);
  if (PARTS) {
    // a thread's first item and group of splits: requested ahead of the factors
    constexpr int PB = 16;
    const int ps = p.K32 + 4, quads = p.ldw / 4, items = rows * quads;
    const int groups = min(max(TH / items, 1), p.nsplit), per = (p.nsplit + groups - 1) / groups;
    const int k = groups > 1 ? tid / items : 0;
    const int s0 = k * per, s1 = min(p.nsplit, s0 + per);  // (none: s1 <= s0)
    auto source = [&](int i) {  // (past the latent: zeros from its padding's product, never used)
      const int m = i / quads, c = min(i % quads * 4, p.K32 - 4);
      return p.parts + ((size_t)(i0 + m) * p.H + h) * p.nsplit * ps + c;
    };
    const int item = groups > 1 ? tid - k * items : min(tid, items - 1);
    floatx4 pre[PB];
    {
      const float* src = source(item);
#pragma unroll
      for (int s = 0; s < PB; ++s) pre[s] = *reinterpret_cast<const floatx4*>(src + (size_t)min(s0 + s, s1 - 1) * ps);
    }
    for (int i = wave; i < rows; i += NW) {
      const float* src = p.parts + ((size_t)(i0 + i) * p.H + h) * p.nsplit * ps + p.K32;
      const bool on = lane < p.nsplit;
      const float m1 = on ? src[(size_t)lane * ps] : -INFINITY, l1 = on ? src[(size_t)lane * ps + 1] : 0.f;
      const float mm = wave_max_f32_uniform(m1);
      const float w1 = m1 == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m1 - mm);
      const float inv = 1.f / wave_sum_uniform(l1 * w1);
      if (on) fac[i][lane] = w1 * inv;
    }
    __syncthreads();
    auto add = [&](floatx4& v, const floatx4& u, int m, int s) {
      const float f = s < s1 ? fac[m][s] : 0.f;
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = fmaf(f, u[e], v[e]);
    };
    auto rest = [&](floatx4& v, int i, int s) {  // splits from s on
      const float* src = source(i);
      for (; s < s1; s += 8) {
        floatx4 u[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) u[e] = *reinterpret_cast<const floatx4*>(src + (size_t)min(s + e, s1 - 1) * ps);
#pragma unroll
        for (int e = 0; e < 8; ++e) add(v, u[e], i / quads, min(s + e, kMaxSplits - 1));
      }
    };
    auto leave = [&](int i, const floatx4& v) {
      const int c = i % quads * 4;
      T* dst = reinterpret_cast<T*>(xs + i / quads * lrow) + c;
#pragma unroll
      for (int e = 0; e < 4; ++e) dst[e] = Elem<T>::make(c < p.K32 ? v[e] : 0.f);
    };
    floatx4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < PB; ++s) add(v, pre[s], item / quads, min(s0 + s, kMaxSplits - 1));
    rest(v, item, s0 + PB);
    if (groups > 1) {  // (then items <= TH / 2)
      if (k < groups) sums[tid] = v;
      __syncthreads();
      if (tid < items) {
        for (int o = 1; o < groups; ++o) v += sums[tid + o * items];
        leave(tid, v);
      }
    } else {
      if (tid < items) leave(tid, v);
      for (int i = tid + TH; i < items; i += TH) {
        floatx4 w = {0.f, 0.f, 0.f, 0.f};
        rest(w, i, 0);
        leave(i, w);
      }
    }
    __syncthreads();
    xp = xs + min(r, rows - 1) * lrow + g * 16;
  }
  floatx4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int s = first; s < steps; s += kHeadBatch) {
    uint4 xv[kHeadBatch];
#pragma unroll
    for (int i = 0; i < kHeadBatch; ++i) xv[i] = load16(xp + min(s + i, all - 1) * 64);
#pragma unroll
    for (int i = 0; i < kHeadBatch; ++i)
      if (s + i < steps) acc = Elem<T>::mma16(wv[i], xv[i], acc);
    if (s + kHeadBatch < steps) load_w(s + kHeadBatch);
  }
  if (KW > 1) {
    red[wave][lane] = acc;
    __syncthreads();
    if (wave % KW) return;
#pragma unroll
    for (int k = 1; k < KW; ++k) acc += red[wave + k][lane];
  }
  if (r >= rows) return;
  T* y = reinterpret_cast<T*>(p.y) + (size_t)row * p.ldy + (size_t)h * p.yh;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (n0 + 4 * g + e < p.N) y[n0 + 4 * g + e] = Elem<T>::make(acc[e]);
}

// ------------------------------------------------------------------------------ expanded
// pages of the pool -> rows: latent [64 n][cp], shared key part [64 n][r8]; zeros behind both
template <typename T>
__global__ __launch_bounds__(256) void latent_gather_kernel(const T* __restrict__ pool, const int32_t* __restrict__ table,
                                                            const int2* __restrict__ pages, T* __restrict__ c, T* __restrict__ k,
                                                            int max_pages, int ldk, int C, int c32, int cp, int rot, int r8) {
  constexpr int VEC = Elem<T>::kVec;
  const int2 pg = pages[blockIdx.x];
  const T* src = pool + (size_t)table[(size_t)pg.x * max_pages + pg.y] * kPage * ldk;
  const int cv = cp / VEC, row0 = blockIdx.y * 16;
  for (int i = threadIdx.x; i < 16 * cv; i += 256) {
    const int row = row0 + i / cv, d = i % cv * VEC;
    const uint4 v = d < c32 ? *reinterpret_cast<const uint4*>(src + (size_t)row * ldk + d) : uint4{0, 0, 0, 0};
    *reinterpret_cast<uint4*>(c + ((size_t)blockIdx.x * kPage + row) * cp + d) = v;
  }
  for (int i = threadIdx.x; i < 16 * r8; i += 256) {
    const int row = row0 + i / r8, d = i % r8;
    k[((size_t)blockIdx.x * kPage + row) * r8 + d] = d < rot ? src[(size_t)row * ldk + c32 + d] : Elem<T>::make(0.f);
  }
}

int check(const exo_latent_attn* a, const char* what) {
  EXO_REQUIRE(a && (a->dtype == 0 || a->dtype == 1), "%s: bad dtype", what);
  EXO_REQUIRE(a->n > 0 && a->n <= 65535 && a->heads > 0 && a->heads <= 65535, "%s: bad counts (n=%d heads=%d)", what, a->n, a->heads);
  EXO_REQUIRE(a->rank > 0 && a->rank <= 512 && a->rot >= 0 && a->rot % 2 == 0 && a->rot <= kMaxRot,
              "%s: latent size %d not in 1..512 or rotated part %d not even and <= %d", what, a->rank, a->rot, kMaxRot);
  EXO_REQUIRE(a->ldk % 32 == 0 && a->ldk >= (a->rank + 31) / 32 * 32 + a->rot && a->ldk <= 640, "%s: pool rows of %d elements", what, a->ldk);
  EXO_REQUIRE(a->q && a->kv && a->gain && (a->freq || !a->rot) && a->pool && a->table && a->slot && a->pos && a->max_pages > 0 &&
                  a->ldkv >= a->rank + a->rot && a->rot_col % 8 == 0 && a->ldq >= a->rot_col + a->heads * ((a->rot + 7) / 8 * 8),
              "%s: null pointer or short rows", what);
  return EXO_OK;
}

template <typename T, int KMAX, bool FUSE>
int launch_rows(const Params& p, hipStream_t st) {
  constexpr int KT = sizeof(T) == 2 ? 64 : 32;
  const int lds = KT * (p.ldk * (int)sizeof(T) + 16) + (sizeof(T) == 2 ? 32 : 16) * kPRow;
  exo_note_variant("latent_rows<%s,%d,%s> splits=%d rows=%d", sizeof(T) == 2 ? "bf16" : "f32", KMAX, FUSE ? "fused" : "plain", p.nsplit, p.n);
  static bool done = false;
  const auto fn = latent_rows_kernel<T, KMAX, FUSE>;
  if (!done) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
    if (e != hipSuccess) {
      exo_set_error("exo_latent_rows: cannot raise the dynamic LDS limit: %s", hipGetErrorString(e));
      return EXO_ERR_HIP;
    }
    done = true;
  }
  fn<<<dim3(p.nsplit, (p.H + p.gsz - 1) / p.gsz, p.n), kRowThreads, lds, st>>>(p);
  return EXO_OK;
}
template <typename T, int KMAX>
int launch_rows_f(const Params& p, bool fuse, hipStream_t st) {
  return fuse ? launch_rows<T, KMAX, true>(p, st) : launch_rows<T, KMAX, false>(p, st);
}
template <typename T>
int launch_rows_k(const Params& p, bool fuse, hipStream_t st) {
  return p.ldk <= 192 ? launch_rows_f<T, 192>(p, fuse, st) : p.ldk <= 320 ? launch_rows_f<T, 320>(p, fuse, st)
         : p.ldk <= 576 ? launch_rows_f<T, 576>(p, fuse, st) : launch_rows_f<T, 640>(p, fuse, st);
}

}  // namespace

extern "C" int exo_latent_prepare(const exo_latent_attn* a, exo_stream_t stream) {
  const int rc = check(a, "exo_latent_prepare");
  if (rc) return rc;
  EXO_REQUIRE(!a->prepared, "exo_latent_prepare: the rows are prepared");
  const Params p = params_of(a);
  const int grid = (p.n + kWaves - 1) / kWaves;
  if (a->dtype == 0)
    latent_prepare_kernel<bf16_t><<<grid, 64 * kWaves, 0, (hipStream_t)stream>>>(p);
  else
    latent_prepare_kernel<float><<<grid, 64 * kWaves, 0, (hipStream_t)stream>>>(p);
  EXO_CHECK_LAUNCH("exo_latent_prepare");
  return EXO_OK;
}

extern "C" int64_t exo_latent_parts(int n, int heads, int rank, int nsplit) {
  return (int64_t)n * heads * nsplit * ((rank + 31) / 32 * 32 + 4);
}

extern "C" int exo_latent_rows(const exo_latent_attn* a, int append, exo_stream_t stream) {
  const int rc = check(a, "exo_latent_rows");
  if (rc) return rc;
  Params p = params_of(a);
  EXO_REQUIRE(a->q_latent && a->ldql >= p.H * p.cp && a->ldql % 8 == 0 && a->nsplit >= 1 && a->nsplit <= kMaxSplits &&
                  (a->nsplit == 1 ? a->out && a->ldo >= p.H * p.cp : a->parts && a->parts_floats >= exo_latent_parts(a->n, a->heads, a->rank, a->nsplit)),
              "exo_latent_rows: bad queries, splits (%d) or output", a->nsplit);
  EXO_REQUIRE(!append || (!a->prepared && !a->list), "exo_latent_rows: rows that append are neither prepared nor listed");
  p.gsz = p.H < 16 ? p.H : 16;
  const hipStream_t st = (hipStream_t)stream;
  const int rc2 = a->dtype == 0 ? launch_rows_k<bf16_t>(p, append != 0, st) : launch_rows_k<float>(p, append != 0, st);
  if (rc2) return rc2;
  EXO_CHECK_LAUNCH("exo_latent_rows");
  return EXO_OK;
}

extern "C" int exo_head_linear(const exo_head_linear_args* a, exo_stream_t stream) {
  EXO_REQUIRE(a && (a->dtype == 0 || a->dtype == 1) && a->w && a->y, "exo_head_linear: bad dtype or null pointer");
  EXO_REQUIRE(a->n > 0 && a->heads > 0 && a->heads <= 65535 && a->N > 0 && a->K > 0 && a->ldw % 64 == 0 && a->ldw >= a->K && a->ldw <= 2048,
              "exo_head_linear: bad sizes (n=%d heads=%d N=%d K=%d ldw=%d)", a->n, a->heads, a->N, a->K, a->ldw);
  EXO_REQUIRE(a->ldy >= (a->heads - 1) * a->y_head + a->N && a->y_head >= a->N, "exo_head_linear: output rows of %d elements", a->ldy);
  const int vec = a->dtype == 0 ? 8 : 4;
  EXO_REQUIRE(a->parts ? a->nsplit >= 1 && a->nsplit <= kMaxSplits && a->ldw <= 512 &&
                             a->parts_floats >= exo_latent_parts(a->n, a->heads, a->K, a->nsplit)
                       : a->x && a->x_head % vec == 0 && a->ldx % vec == 0 && a->ldx >= (a->heads - 1) * a->x_head + a->ldw,
              "exo_head_linear: bad operand (rows of %d, %d per head)", a->ldx, a->x_head);
  HeadLinear p{};
  p.x = a->x, p.parts = a->parts, p.w = a->w, p.y = a->y, p.list = a->list, p.n = a->n, p.H = a->heads, p.N = a->N;
  p.K32 = (a->K + 31) / 32 * 32, p.ldx = a->ldx, p.xh = a->x_head, p.ldw = a->ldw, p.ldy = a->ldy, p.yh = a->y_head, p.nsplit = a->nsplit;
  const int threads = p.parts ? 512 : 256;
  const dim3 grid(exo_ceil_div(p.N, p.parts ? 32 : 64), p.H, exo_ceil_div(p.n, 16));
  EXO_REQUIRE(grid.z <= 65535, "exo_head_linear: too many rows (%d)", p.n);
  const int lds = p.parts ? (p.n < 16 ? p.n : 16) * (p.ldw * (a->dtype == 0 ? 2 : 4) + 16) : 0;
  const hipStream_t st = (hipStream_t)stream;
  if (p.parts) {
    if (a->dtype == 0)
      head_linear_kernel<bf16_t, true><<<grid, threads, lds, st>>>(p);
    else
      head_linear_kernel<float, true><<<grid, threads, lds, st>>>(p);
  } else if (a->dtype == 0) {
    head_linear_kernel<bf16_t, false><<<grid, threads, 0, st>>>(p);
  } else {
    head_linear_kernel<float, false><<<grid, threads, 0, st>>>(p);
  }
  EXO_CHECK_LAUNCH("exo_head_linear");
  return EXO_OK;
}

extern "C" int exo_latent_gather(const exo_latent_attn* a, const int32_t* pages, int n_pages, void* c, void* k, exo_stream_t stream) {
  const int rc = check(a, "exo_latent_gather");
  if (rc) return rc;
  EXO_REQUIRE(a->dtype == 0 && pages && n_pages > 0 && c && k, "exo_latent_gather: bf16 only, null pointer or no pages");
  const Params p = params_of(a);
  latent_gather_kernel<bf16_t><<<dim3(n_pages, kPage / 16), 256, 0, (hipStream_t)stream>>>(
      (const bf16_t*)p.pool, p.table, (const int2*)pages, (bf16_t*)c, (bf16_t*)k, p.max_pages, p.ldk, p.C, p.c32, p.cp, p.rot, p.r8);
  EXO_CHECK_LAUNCH("exo_latent_gather");
  return EXO_OK;
}
