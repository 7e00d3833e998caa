// Products with unquantised matrices: y[M,N] = x[M,K] @ w[N,K]^T (+ bias), element type bf16 or
// float, float32 accumulation.  Row strides are multiples of 64 elements and the columns between
// K and the stride are zero in BOTH operands, so no kernel has a K tail and any K is taken.
//
//  * dense_gemv_kernel, up to 16 rows of x: 16 weight rows per workgroup, K dealt out over its
//    waves, weights straight from memory into the A operand of a 16x16 matrix product (16 rows x
//    64 bytes per load instruction), x rows as the 16 columns of B.  One batch of kBatch loads per
//    wave is in flight before anything is waited for.  Range-checked loads stand in for every
//    tail: rows past N, x rows past M and steps past a wave's range read as zero.
//  * dense_gemm_kernel, any number of rows: a (64 MI) x (64 NJ) tile per workgroup of four waves
//    (2 x 2, each (32 MI) x (32 NJ) in 32x32 products), K steps of 128 bytes per row through two
//    LDS buffers, the next two steps' vectors in registers meanwhile; one barrier per step.  A row's
//    eight 16-byte chunks sit at slot chunk ^ (row % 8), so operand reads of 32 rows meet no bank
//    twice.  PAIR: the weight tile holds rows of a gate and an up matrix, 32 and 32, so that a
//    wave's column tiles are (gate, up) of the same outputs and the gated unit is its epilogue.
//    GROUPED: the rows are one expert's (token, slot) pairs, from exo_moe_group's tile list.
#include "../../include/exo_mi355x.h"
#include "dense.h"

namespace {

// ------------------------------------------------------------------------------ GEMV
constexpr int kBatch = 8;

struct GemvParams {
  const void* x;
  const void* w;
  const float* bias;
  void* y;
  int M, N, ldx, ldw, ldy, y_f32;
};

template <typename T>
__device__ __forceinline__ void store_out(void* y, size_t i, float v, int y_f32) {
  if (y_f32)
    reinterpret_cast<float*>(y)[i] = v;
  else
    reinterpret_cast<T*>(y)[i] = Elem<T>::make(v);
}

// Norm of the previous sublayer's output and residual sum, in front of the product that reads the
// residual: every workgroup forms x + gain * branch / rms(branch) for itself (in LDS, element type),
// workgroup 0 also writes it out - to another buffer than it is read from, since the others may
// still be reading.
struct PostNorm {
  const float* x;       // [M][H]
  const float* branch;  // [M][H]
  const float* gain;    // [H]
  float* x_out;         // [M][H]
  void* xb_out;         // T [M][ldx], or null
  int H;
  float eps;
};
constexpr int kPostPasses = 4;  // float4 per lane of a row's waves

__host__ __device__ inline int post_waves_per_row(int M, int NW) {
  int p = 1;
  while (p < M) p *= 2;
  return NW > p ? NW / p : 1;
}

template <typename T, int NW, bool POST>
__global__ __launch_bounds__(64 * NW) void dense_gemv_kernel(const GemvParams p, const PostNorm q) {
  __shared__ float red[NW][256];
  __shared__ float part[NW];
  extern __shared__ __attribute__((aligned(16))) char xs[];  // POST: [M][ldx * sizeof(T) + 16]
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane((int)threadIdx.x >> 6);
  const int r = lane & 15, g = lane >> 4;
  const int n0 = blockIdx.x * 16, rows = min(16, p.N - n0);
  const uint32_t wrow = (uint32_t)p.ldw * sizeof(T), xrow = (uint32_t)p.ldx * sizeof(T);
  const int steps = (int)(wrow >> 6);
  const int per = (steps + NW - 1) / NW, s0 = min(steps, wave * per), s1 = min(steps, s0 + per);
  const __amdgpu_buffer_rsrc_t rw =
      buf_of(reinterpret_cast<const char*>(p.w) + (size_t)n0 * wrow, (uint32_t)rows * wrow);
  const __amdgpu_buffer_rsrc_t rx = buf_of(p.x, (uint32_t)p.M * xrow);
  const uint32_t woff = r * wrow + g * 16;
  uint4 wv[kBatch];
  auto load_w = [&](int s) {
#pragma unroll
    for (int i = 0; i < kBatch; ++i) wv[i] = buf_load16(rw, s + i < s1 ? woff + (s + i) * 64 : kPastEnd, 0);
  };
  if (POST) {
    // a row's columns over wpr waves; its inputs are requested ahead of the first weights
    const int wpr = post_waves_per_row(p.M, NW), rpi = NW / wpr;  // rows per iteration
    const uint32_t lrow = xrow + 16;
    const bool vec = q.H % 4 == 0;
    for (int m0 = 0; m0 < p.M; m0 += rpi) {
      const int m = m0 + wave / wpr, c0 = ((wave % wpr) * 64 + lane) * 4, cs = wpr * 256;
      floatx4 v[kPostPasses], x[kPostPasses], gn[kPostPasses];
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < kPostPasses; ++i) {
        const int c = c0 + i * cs;
        v[i] = x[i] = gn[i] = floatx4{0.f, 0.f, 0.f, 0.f};
        if (m < p.M && c < q.H) {
          const size_t o = (size_t)m * q.H + c;
          if (vec) {
            v[i] = *reinterpret_cast<const floatx4*>(q.branch + o);
            x[i] = *reinterpret_cast<const floatx4*>(q.x + o);
            gn[i] = *reinterpret_cast<const floatx4*>(q.gain + c);
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (c + e < q.H) v[i][e] = q.branch[o + e], x[i][e] = q.x[o + e], gn[i][e] = q.gain[c + e];
          }
        }
      }
      if (m0 == 0) load_w(s0);
#pragma unroll
      for (int i = 0; i < kPostPasses; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) ss += v[i][e] * v[i][e];
      ss = wave_sum(ss);
      __syncthreads();  // (the sums of an earlier iteration have been read)
      if (lane == 0) part[wave] = ss;
      __syncthreads();
      float tot = 0.f;
      for (int w = 0; w < wpr; ++w) tot += part[wave / wpr * wpr + w];
      const float inv = 1.f / sqrtf(tot / q.H + q.eps);
#pragma unroll
      for (int i = 0; i < kPostPasses; ++i) {
        const int c = c0 + i * cs;
        if (m >= p.M || c >= p.ldx) continue;
        T out[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float y = x[i][e] + v[i][e] * inv * gn[i][e];  // zero past H
          out[e] = Elem<T>::make(y);
          if (blockIdx.x == 0 && c + e < q.H) {
            q.x_out[(size_t)m * q.H + c + e] = y;
            if (q.xb_out) reinterpret_cast<T*>(q.xb_out)[(size_t)m * p.ldx + c + e] = out[e];
          }
        }
        T* dst = reinterpret_cast<T*>(xs + m * lrow) + c;
#pragma unroll
        for (int e = 0; e < 4; ++e) dst[e] = out[e];
      }
    }
    __syncthreads();
  } else {
    load_w(s0);
  }
  floatx4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int s = s0; s < s1; s += kBatch) {
    uint4 xv[kBatch];
#pragma unroll
    for (int i = 0; i < kBatch; ++i) {
      if (POST)  // (steps past the range: any finite values, their weights are zero)
        xv[i] = *reinterpret_cast<const uint4*>(xs + min(r, p.M - 1) * (xrow + 16) + g * 16 + min(s + i, s1 - 1) * 64);
      else
        xv[i] = buf_load16(rx, s + i < s1 ? r * xrow + g * 16 + (s + i) * 64 : kPastEnd, 0);
    }
#pragma unroll
    for (int i = 0; i < kBatch; ++i) acc = Elem<T>::mma16(wv[i], xv[i], acc);
    if (s + kBatch < s1) load_w(s + kBatch);
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) red[wave][r * 16 + 4 * g + e] = acc[e];  // [m][n]
  __syncthreads();
  for (int o = threadIdx.x; o < 16 * p.M; o += 64 * NW) {
    const int m = o >> 4, n = o & 15;
    if (n >= rows) continue;
    float v = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) v += red[w][o];
    if (p.bias) v += p.bias[n0 + n];
    store_out<T>(p.y, (size_t)m * p.ldy + n0 + n, v, p.y_f32);
  }
}

// ------------------------------------------------------------------------------ GEMM
struct GemmParams {
  const void* x;
  const void* w;   // gate matrix in pair mode
  const void* w2;  // up matrix
  const float* bias;
  void* y;
  int M, N, ldx, ldw, ldy, y_f32;
  GluConst glu;
  // grouped
  const int32_t* sorted;
  const int32_t* tiles;
  int x_div;           // x row of a pair = pair / x_div
  size_t w_stride;     // elements between experts
  // split over K
  int ksplit, ksteps;  // 128-byte steps per split
  float* part;         // [ksplit][M][N]
};

template <typename T, int MI, int NJ, bool GROUPED, bool PAIR>
__global__ __launch_bounds__(256, 2) void dense_gemm_kernel(const GemmParams p) {
  constexpr int BM = 64 * MI, BW = 64 * NJ;      // tile rows of x, of weights
  constexpr int BN = PAIR ? BW / 2 : BW;         // output columns
  constexpr int XV = BM * 8 / 256, WV = BW * 8 / 256;
  constexpr int PD = 2;
  extern __shared__ __attribute__((aligned(16))) char lds[];  // [2][(BM + BW) * 128]
  __shared__ int row_pair[GROUPED ? BM : 1];
  constexpr int BUF = (BM + BW) * 128;

  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wm = (wave >> 1) * (32 * MI), wn = (wave & 1) * (32 * NJ);
  // Consecutive workgroups go to different XCDs: give each XCD a contiguous run of tiles, row
  // tiles innermost, so that it streams few weight columns through its own L2.
  int bx, by;
  {
    const int total = (int)(gridDim.x * gridDim.y), id = (int)(blockIdx.y * gridDim.x + blockIdx.x);
    const int q = total >> 3, rem = total & 7, xcd = id & 7, k = id >> 3;
    const int t = xcd * q + min(xcd, rem) + k;
    by = t % (int)gridDim.y;
    bx = t / (int)gridDim.y;
  }
  const int n0 = bx * BN;
  int m0 = by * BM, m_end = p.M;
  size_t w_off = 0;
  if (GROUPED) {
    const int32_t* ti = p.tiles + 3 * (size_t)by;
    const int e = ti[0];
    if (e < 0) return;  // whole workgroup: an unused entry of the tile list
    m0 = 0;
    m_end = ti[2];
    for (int i = tid; i < BM; i += 256) row_pair[i] = p.sorted[ti[1] + min(i, m_end - 1)];
    w_off = (size_t)e * p.w_stride * sizeof(T);
    __syncthreads();
  }
  const uint32_t wrow = (uint32_t)p.ldw * sizeof(T), xrow = (uint32_t)p.ldx * sizeof(T);
  const int all_steps = (int)(wrow >> 7);
  const int k0 = p.ksplit > 1 ? (int)blockIdx.z * p.ksteps : 0;
  const int steps = (p.ksplit > 1 ? min(all_steps, k0 + p.ksteps) : all_steps) - k0;

  const char* xbase = reinterpret_cast<const char*>(p.x);
  if (!GROUPED) xbase += (size_t)m0 * xrow;
  const char* wbase = reinterpret_cast<const char*>(p.w) + w_off + (size_t)n0 * wrow;
  const uint32_t wbytes = (uint32_t)min(BN, p.N - n0) * wrow;  // rows past N read as zero
  const __amdgpu_buffer_rsrc_t rx = buf_of(xbase, 0xFFFFFFFFu);
  __amdgpu_buffer_rsrc_t rw[PAIR ? 2 : 1];
  rw[0] = buf_of(wbase, wbytes);
  if (PAIR)
    rw[PAIR ? 1 : 0] = buf_of(reinterpret_cast<const char*>(p.w2) + w_off + (size_t)n0 * wrow, wbytes);
  uint32_t xoff[XV], woff[WV];
#pragma unroll
  for (int i = 0; i < XV; ++i) {
    const int id = tid + 256 * i, tr = id >> 3, c = id & 7;
    const uint32_t row = GROUPED ? (uint32_t)(row_pair[tr] / p.x_div) : (uint32_t)min(tr, m_end - 1 - m0);
    xoff[i] = row * xrow + c * 16;
  }
#pragma unroll
  for (int i = 0; i < WV; ++i) {
    const int id = tid + 256 * i, tr = id >> 3, c = id & 7;
    // A pass of 256 threads covers one 32-row tile of the weight block: tile i belongs to wave
    // column half i / NJ.  PAIR: its column tiles alternate gate / up over the same 32 outputs.
    const int n = PAIR ? (i / NJ) * (16 * NJ) + ((i % NJ) >> 1) * 32 + (tr & 31) : tr;
    woff[i] = (uint32_t)n * wrow + c * 16;
  }
  // PD steps of tiles in flight in registers.  Requests past the last step re-read it: every load
  // is unconditional, so the waits count exactly the loads in front of the ones they are for.
  uint4 xr[PD][XV], wr[PD][WV];
  auto load_regs = [&](uint4 (&x)[XV], uint4 (&w)[WV], int s) {
    const uint32_t so = (uint32_t)(k0 + min(s, steps - 1)) * 128;
#pragma unroll
    for (int i = 0; i < XV; ++i) x[i] = buf_load16(rx, xoff[i], so);
#pragma unroll
    for (int i = 0; i < WV; ++i) w[i] = buf_load16(rw[PAIR ? (i % NJ) & 1 : 0], woff[i], so);
  };
  auto store_lds = [&](const uint4 (&x)[XV], const uint4 (&w)[WV], int b) {
    char* xl = lds + b * BUF;
    char* wl = xl + BM * 128;
#pragma unroll
    for (int i = 0; i < XV; ++i) {
      const int id = tid + 256 * i, tr = id >> 3, c = id & 7;
      *reinterpret_cast<uint4*>(xl + tr * 128 + ((c ^ (tr & 7)) << 4)) = x[i];
    }
#pragma unroll
    for (int i = 0; i < WV; ++i) {
      const int id = tid + 256 * i, tr = id >> 3, c = id & 7;
      *reinterpret_cast<uint4*>(wl + tr * 128 + ((c ^ (tr & 7)) << 4)) = w[i];
    }
  };
  const int frow = lane & 31, half = lane >> 5;
  floatx16 acc[MI][NJ];
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < NJ; ++j)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[i][j][e] = 0.f;

#pragma unroll
  for (int u = 0; u < PD; ++u) load_regs(xr[u], wr[u], u);
  store_lds(xr[0], wr[0], 0);
  load_regs(xr[0], wr[0], PD);
  for (int s0 = 0; s0 < steps; s0 += PD) {
#pragma unroll
    for (int u = 0; u < PD; ++u) {
      const int s = s0 + u;
      if (s >= steps) break;
      __syncthreads();  // step s is complete in its buffer, the other buffer is no longer read
      const int v = (u + 1) % PD;
      store_lds(xr[v], wr[v], (s + 1) & 1);
      load_regs(xr[v], wr[v], s + 1 + PD);
      __builtin_amdgcn_sched_barrier(0);  // (left alone, the requests sink behind the products)
      const char* xl = lds + (s & 1) * BUF + (wm + frow) * 128;
      const char* wl = lds + (s & 1) * BUF + (BM + wn + frow) * 128;
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        const int slot = ((2 * t + half) ^ (frow & 7)) << 4;
        uint4 a[MI], b[NJ];
#pragma unroll
        for (int i = 0; i < MI; ++i) a[i] = *reinterpret_cast<const uint4*>(xl + i * 4096 + slot);
#pragma unroll
        for (int j = 0; j < NJ; ++j) b[j] = *reinterpret_cast<const uint4*>(wl + j * 4096 + slot);
#pragma unroll
        for (int i = 0; i < MI; ++i)
#pragma unroll
          for (int j = 0; j < NJ; ++j) acc[i][j] = Elem<T>::mma32(a[i], b[j], acc[i][j]);
      }
    }
  }

  // ---- epilogue: element e of tile (i, j): row wm + 32 i + 8 (e / 4) + 4 half + e % 4, column lane
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int tr = wm + 32 * i + 8 * (e >> 2) + 4 * half + (e & 3);
      if (m0 + tr >= m_end) continue;
      const size_t row = GROUPED ? (size_t)row_pair[tr] : (size_t)(m0 + tr);
      if (PAIR) {
#pragma unroll
        for (int j = 0; j < NJ; j += 2) {
          const int n = n0 + (wave & 1) * (16 * NJ) + (j >> 1) * 32 + frow;
          if (n < p.N)
            reinterpret_cast<T*>(p.y)[row * p.ldy + n] =
                Elem<T>::make(clamped_glu(acc[i][j][e], acc[i][j + 1 < NJ ? j + 1 : j][e], p.glu));
        }
      } else {
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
          const int n = n0 + wn + 32 * j + frow;
          if (n >= p.N) continue;
          if (p.ksplit > 1) {
            p.part[((size_t)blockIdx.z * p.M + row) * p.N + n] = acc[i][j][e];
          } else {
            const float v = acc[i][j][e] + (p.bias ? p.bias[n] : 0.f);
            store_out<T>(p.y, row * p.ldy + n, v, p.y_f32);
          }
        }
      }
    }
}

// adds the K ranges in their order
template <typename T>
__global__ __launch_bounds__(256) void dense_reduce_kernel(const GemmParams p) {
  const int n = blockIdx.x * 256 + threadIdx.x, m = blockIdx.y;
  if (n >= p.N) return;
  float v = p.bias ? p.bias[n] : 0.f;
  for (int z = 0; z < p.ksplit; ++z) v += p.part[((size_t)z * p.M + m) * p.N + n];
  store_out<T>(p.y, (size_t)m * p.ldy + n, v, p.y_f32);
}

int raise_lds(const void* fn, int bytes, bool* done) {
  if (*done || bytes <= 64 * 1024) return EXO_OK;
  const hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
  if (e != hipSuccess) {
    exo_set_error("cannot raise the dynamic LDS limit to %d bytes: %s", bytes, hipGetErrorString(e));
    return EXO_ERR_HIP;
  }
  *done = true;
  return EXO_OK;
}

template <typename T, int MI, int NJ, bool GROUPED, bool PAIR>
int launch_gemm(const GemmParams& p, int row_tiles, hipStream_t st) {
  constexpr int lds = 2 * (64 * MI + 64 * NJ) * 128;
  static bool done = false;
  const auto fn = dense_gemm_kernel<T, MI, NJ, GROUPED, PAIR>;
  const int rc = raise_lds(reinterpret_cast<const void*>(fn), lds, &done);
  if (rc) return rc;
  const int bn = PAIR ? 32 * NJ : 64 * NJ;
  const dim3 grid(exo_ceil_div(p.N, bn), row_tiles, p.ksplit);
  exo_note_variant("dense_gemm<%s,%d,%d,%s,%s> grid=%dx%dx%d", sizeof(T) == 2 ? "bf16" : "f32", MI, NJ,
                   GROUPED ? "grouped" : "plain", PAIR ? "pair" : "single", (int)grid.x, (int)grid.y, (int)grid.z);
  fn<<<grid, 256, lds, st>>>(p);
  return EXO_OK;
}

// rows per tile: the tallest that still leaves a workgroup per CU, else the shorter ones
template <typename T, bool PAIR>
int launch_plain(GemmParams p, int64_t ws_floats, hipStream_t st) {
  const int cols = exo_ceil_div(p.N, PAIR ? 64 : 128);
  const int steps = (int)((int64_t)p.ldw * sizeof(T) / 128);
  p.ksplit = 1;
  p.ksteps = steps;
  const int64_t t2 = (int64_t)cols * exo_ceil_div(p.M, 128), t1 = (int64_t)cols * exo_ceil_div(p.M, 64);
  const bool tall = p.M > 64 && t2 >= 192;
  if (!PAIR && p.part) {  // few tiles: split K until the chip has about one workgroup per CU
    const int64_t tiles = tall ? t2 : t1;
    int ks = 1;
    while (ks < 16 && tiles * ks * 2 <= 256 && steps / (ks * 2) >= 4) ks *= 2;
    while (ks > 1 && (int64_t)ks * p.M * p.N > ws_floats) ks /= 2;
    if (ks > 1) {
      p.ksteps = exo_ceil_div(steps, ks);
      p.ksplit = exo_ceil_div(steps, p.ksteps);
    }
  }
  int rc;
  if (tall)
    rc = launch_gemm<T, 2, 2, false, PAIR>(p, exo_ceil_div(p.M, 128), st);
  else
    rc = launch_gemm<T, 1, 2, false, PAIR>(p, exo_ceil_div(p.M, 64), st);
  if (rc) return rc;
  if (p.ksplit > 1)
    dense_reduce_kernel<T><<<dim3(exo_ceil_div(p.N, 256), p.M), 256, 0, st>>>(p);
  return EXO_OK;
}

int gemv_waves(int N) {
  const int tiles = exo_ceil_div(N, 16);
  return tiles >= 1024 ? 4 : tiles >= 256 ? 8 : 16;
}
// the columns of a row fit its waves' registers, the rows fit the LDS
bool post_fits(int M, int N, int H, int ldx, int elem) {
  return M <= 16 && ldx <= post_waves_per_row(M, gemv_waves(N)) * 256 * kPostPasses && H <= ldx &&
         (int64_t)M * (ldx * elem + 16) <= 40 * 1024;
}

template <typename T, int NW>
void launch_gemv_nw(const GemvParams& p, const PostNorm* q, hipStream_t st) {
  const int tiles = exo_ceil_div(p.N, 16);
  if (q)
    dense_gemv_kernel<T, NW, true><<<tiles, 64 * NW, p.M * (p.ldx * (int)sizeof(T) + 16), st>>>(p, *q);
  else
    dense_gemv_kernel<T, NW, false><<<tiles, 64 * NW, 0, st>>>(p, PostNorm{});
}
template <typename T>
int launch_gemv(const GemvParams& p, const PostNorm* q, hipStream_t st) {
  const int nw = gemv_waves(p.N);
  exo_note_variant("dense_gemv<%s,%d,%s> M=%d N=%d", sizeof(T) == 2 ? "bf16" : "f32", nw, q ? "post" : "plain", p.M, p.N);
  if (nw == 4)
    launch_gemv_nw<T, 4>(p, q, st);
  else if (nw == 8)
    launch_gemv_nw<T, 8>(p, q, st);
  else
    launch_gemv_nw<T, 16>(p, q, st);
  return EXO_OK;
}

#define EXO_DENSE_ARGS(what)                                                                            \
  EXO_REQUIRE(dtype == 0 || dtype == 1, what ": dtype must be 0 (bf16) or 1 (float32)");                \
  EXO_REQUIRE(x && w && y, what ": null pointer");                                                      \
  EXO_REQUIRE(M > 0 && N > 0 && ldx > 0 && ldx == ldw && ldw % 64 == 0,                                 \
              what ": need M, N > 0 and equal row strides that are multiples of 64 (got M=%d N=%d %d/%d)", \
              M, N, ldx, ldw);                                                                          \
  EXO_REQUIRE((((uintptr_t)x | (uintptr_t)w) & 15) == 0, what ": operands must be 16-byte aligned");    \
  EXO_REQUIRE((int64_t)ldw * 256 * 4 < (1ll << 31), what ": row stride %d too large", ldw)

}  // namespace

extern "C" int exo_dense_gemv(const void* x, const void* w, const float* bias, void* y, int y_f32, int M, int N,
                              int ldx, int ldw, int ldy, int dtype, exo_stream_t stream) {
  EXO_DENSE_ARGS("exo_dense_gemv");
  EXO_REQUIRE(M <= 16 && ldy >= N, "exo_dense_gemv: M=%d must be <= 16 and ldy=%d >= N=%d", M, ldy, N);
  const GemvParams p{x, w, bias, y, M, N, ldx, ldw, ldy, y_f32};
  const int rc = EXO_BY_TYPE(dtype, launch_gemv<bf16_t>(p, nullptr, (hipStream_t)stream),
                             launch_gemv<float>(p, nullptr, (hipStream_t)stream));
  if (rc) return rc;
  EXO_CHECK_LAUNCH("exo_dense_gemv");
  return EXO_OK;
}

extern "C" int exo_post_gemv_fits(int M, int N, int H, int ldx, int dtype) {
  return M > 0 && N > 0 && H > 0 && post_fits(M, N, H, ldx, dtype == 0 ? 2 : 4);
}

extern "C" int exo_post_gemv(const float* x, const float* branch, const float* gain, float eps, float* x_out,
                             void* xb_out, const void* w, const float* bias, void* y, int y_f32, int M, int N, int H,
                             int ldx, int ldw, int ldy, int dtype, exo_stream_t stream) {
  EXO_DENSE_ARGS("exo_post_gemv");
  EXO_REQUIRE(branch && gain && x_out && x_out != x && ldy >= N, "exo_post_gemv: null pointer, x_out == x or bad ldy");
  EXO_REQUIRE(post_fits(M, N, H, ldx, dtype == 0 ? 2 : 4), "exo_post_gemv: %d rows of %d columns do not fit one launch", M, H);
  const GemvParams p{nullptr, w, bias, y, M, N, ldx, ldw, ldy, y_f32};
  const PostNorm q{x, branch, gain, x_out, xb_out, H, eps};
  const int rc = EXO_BY_TYPE(dtype, launch_gemv<bf16_t>(p, &q, (hipStream_t)stream), launch_gemv<float>(p, &q, (hipStream_t)stream));
  if (rc) return rc;
  EXO_CHECK_LAUNCH("exo_post_gemv");
  return EXO_OK;
}

extern "C" int exo_dense_gemm(const void* x, const void* w, const float* bias, void* y, int y_f32, float* workspace,
                              int64_t workspace_floats, int M, int N, int ldx, int ldw, int ldy, int dtype,
                              exo_stream_t stream) {
  EXO_DENSE_ARGS("exo_dense_gemm");
  EXO_REQUIRE(ldy >= N && M <= 65535 * 64, "exo_dense_gemm: bad ldy=%d or M=%d", ldy, M);
  GemmParams p{};
  p.x = x, p.w = w, p.bias = bias, p.y = y, p.M = M, p.N = N, p.ldx = ldx, p.ldw = ldw, p.ldy = ldy, p.y_f32 = y_f32;
  p.part = workspace;
  const int rc = EXO_BY_TYPE(dtype, (launch_plain<bf16_t, false>(p, workspace_floats, (hipStream_t)stream)),
                             (launch_plain<float, false>(p, workspace_floats, (hipStream_t)stream)));
  if (rc) return rc;
  EXO_CHECK_LAUNCH("exo_dense_gemm");
  return EXO_OK;
}

extern "C" int exo_dense_glu_gemm(const void* x, const void* w, const void* w_up, void* y, float limit, float alpha,
                                  float shift, int M, int N, int ldx, int ldw, int ldy, int dtype,
                                  exo_stream_t stream) {
  EXO_DENSE_ARGS("exo_dense_glu_gemm");
  EXO_REQUIRE(w_up && ldy >= N && M <= 65535 * 64, "exo_dense_glu_gemm: bad w_up, ldy=%d or M=%d", ldy, M);
  GemmParams p{};
  p.x = x, p.w = w, p.w2 = w_up, p.y = y, p.M = M, p.N = N, p.ldx = ldx, p.ldw = ldw, p.ldy = ldy;
  p.glu = GluConst{limit, alpha, shift};
  const int rc = EXO_BY_TYPE(dtype, (launch_plain<bf16_t, true>(p, 0, (hipStream_t)stream)),
                             (launch_plain<float, true>(p, 0, (hipStream_t)stream)));
  if (rc) return rc;
  EXO_CHECK_LAUNCH("exo_dense_glu_gemm");
  return EXO_OK;
}

// Experts of a prompt: x rows by (token, slot) pair through exo_moe_group's workspace.  w_up null:
// the plain product, else the gated pair.  y row = pair index.
extern "C" int exo_dense_grouped_gemm(const void* x, const void* w, const void* w_up, const void* group_ws, void* y,
                                      float limit, float alpha, float shift, int T, int topk, int x_per_pair, int E,
                                      int N, int ldx, int ldw, int ldy, int dtype, exo_stream_t stream) {
  const int M = T;
  EXO_DENSE_ARGS("exo_dense_grouped_gemm");
  EXO_REQUIRE(group_ws && topk > 0 && E > 0 && ldy >= N && (int64_t)T * topk < (1ll << 30),
              "exo_dense_grouped_gemm: bad arguments (T=%d topk=%d E=%d)", T, topk, E);
  EXO_REQUIRE((int64_t)T * (x_per_pair ? topk : 1) * ldx * (dtype ? 4 : 2) < (1ll << 32),
              "exo_dense_grouped_gemm: activations exceed 32-bit byte offsets");
  const int64_t pairs = (int64_t)T * topk;
  const int tiles = (int)((pairs + 127) / 128) + E;  // exo_moe_group's list length
  EXO_REQUIRE(tiles <= 65535, "exo_dense_grouped_gemm: %d row tiles exceed the grid limit", tiles);
  GemmParams p{};
  p.x = x, p.w = w, p.w2 = w_up, p.y = y, p.M = T, p.N = N, p.ldx = ldx, p.ldw = ldw, p.ldy = ldy;
  p.glu = GluConst{limit, alpha, shift};
  p.sorted = reinterpret_cast<const int32_t*>(group_ws);
  p.tiles = p.sorted + pairs;
  p.x_div = x_per_pair ? 1 : topk;
  p.w_stride = (size_t)N * ldw;
  p.ksplit = 1;
  const hipStream_t st = (hipStream_t)stream;
  int rc;
  if (w_up)
    rc = EXO_BY_TYPE(dtype, (launch_gemm<bf16_t, 2, 2, true, true>(p, tiles, st)),
                     (launch_gemm<float, 2, 2, true, true>(p, tiles, st)));
  else
    rc = EXO_BY_TYPE(dtype, (launch_gemm<bf16_t, 2, 2, true, false>(p, tiles, st)),
                     (launch_gemm<float, 2, 2, true, false>(p, tiles, st)));
  if (rc) return rc;
  EXO_CHECK_LAUNCH("exo_dense_grouped_gemm");
  return EXO_OK;
}
