// kernels_lin.hip -- matrix products of layered models on fragment-packed bf16 weights (seq_device.h), and the packing itself.
//
//   lin_kernel      prompts: 128 features x 128 rows per workgroup, 4 waves of 64 x 64, both operands through LDS in fragment
//                   order (global_load_lds, 16 bytes per lane: LDS reads are lane-linear, no bank conflicts), two buffers
//   lin_big_kernel  the same with 256 x 256 and a ring of four stages, where there are enough of such tiles (bf16)
//   few_kernel      up to 16 rows (decoding): 4 waves share 16 features and split k; weights stream from HBM straight into the
//                   MFMA operand registers, 1 KiB contiguous per wave and load
// Both take plain products and the experts' (rows gathered per expert); a launch of few_kernel can hold several products.
#include "layered_kernels.h"
#include "seq_device.h"

#include <math.h>

#include <algorithm>

typedef const __attribute__((address_space(1))) void* gptr;
typedef __attribute__((address_space(3))) void* lptr;

static int cdiv(int a, int b) { return (a + b - 1) / b; }

// ---- packing -----------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void pack_kernel(const uint16_t* __restrict__ src, int rows, int k, uint16_t* __restrict__ dst, int kt, int row0, int col0,
                                                   int interleave, int transpose) {
  const size_t n = (size_t)rows * k;
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) {
    const int r = (int)(transpose ? i % k : i / k), c = (int)(transpose ? i / k : i % k) + col0;
    const int tile = interleave >= 0 ? 2 * (r >> 4) + interleave : (r + row0) >> 4;
    const int rr = interleave >= 0 ? r & 15 : (r + row0) & 15;
    dst[((size_t)tile * kt + (c >> 5)) * 512 + (((c & 31) >> 3) * 16 + rr) * 8 + (c & 7)] = src[i];
  }
}
int launch_pack(hipStream_t st, const uint16_t* src, int rows, int k, uint16_t* dst, int kt, int row0, int col0, int interleave, bool transpose) {
  const size_t n = (size_t)rows * k;
  hipLaunchKernelGGL(pack_kernel, dim3((unsigned)((n + 2047) / 2048)), dim3(256), 0, st, src, rows, k, dst, kt, row0, col0, interleave, (int)transpose);
  return DSK_OK;
}
__global__ __launch_bounds__(256) void widen_kernel(const uint16_t* __restrict__ src, float* __restrict__ dst, size_t n) {
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256)
    dst[i] = __builtin_bit_cast(float, (unsigned)src[i] << 16);
}
int launch_widen(hipStream_t st, const uint16_t* src, float* dst, size_t n) {
  hipLaunchKernelGGL(widen_kernel, dim3((unsigned)((n + 1023) / 1024)), dim3(256), 0, st, src, dst, n);
  return DSK_OK;
}
__global__ __launch_bounds__(256) void exp_kernel(float* __restrict__ x, int n) {
  for (int i = threadIdx.x; i < n; i += 256) x[i] = expf(x[i]);
}
int launch_exp(hipStream_t st, float* x, int n) {
  hipLaunchKernelGGL(exp_kernel, dim3(1), dim3(256), 0, st, x, n);
  return DSK_OK;
}
DEV float random_pm1(uint64_t seed, size_t i) {  // splitmix64 of the index
  uint64_t z = seed + (i + 1) * 0x9E3779B97F4A7C15ull;
  z = (z ^ (z >> 30)) * 0xBF58476D1CE4E5B9ull;
  z = (z ^ (z >> 27)) * 0x94D049BB133111EBull;
  z ^= z >> 31;
  return (float)(int)(z >> 40) * (2.f / 16777216.f) - 1.f;
}
template <typename D>
__global__ __launch_bounds__(256) void random_kernel(D* __restrict__ dst, size_t n, float scale, uint64_t seed) {
  for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (size_t)gridDim.x * 256) dst[i] = (D)(scale * random_pm1(seed, i));
}
int launch_fill_random(hipStream_t st, uint16_t* dst, size_t n, float scale, uint64_t seed) {
  if (n) hipLaunchKernelGGL(random_kernel<bf16>, dim3(4096), dim3(256), 0, st, reinterpret_cast<bf16*>(dst), n, scale, seed);
  return DSK_OK;
}
int launch_fill_random_f32(hipStream_t st, float* dst, size_t n, float scale, uint64_t seed) {
  if (n) hipLaunchKernelGGL(random_kernel<float>, dim3(256), dim3(256), 0, st, dst, n, scale, seed);
  return DSK_OK;
}

// ---- epilogues: four consecutive features of one row, out of one lane's accumulator ----------------
DEV float glu(float g, float u, float limit, float alpha, float offset) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f(alpha * g) * (u + offset);
}
template <typename T>
DEV void store_plain(const LinArgs& a, int row, int feature, f32x4 v) {
  typedef typename Frag<T>::four four;
  if (a.epi == LIN_SOFTCAP) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = a.p0 * tanhf(v[i] / a.p0);
  } else if (a.epi == LIN_SCALE) {
    v *= a.p0;
  } else if (a.epi == LIN_XIELU) {
#pragma unroll
    for (int i = 0; i < 4; ++i)  // (exp(z) - 1 - z: its absolute error is a rounding of 1, and z / 2 is beside it)
      v[i] = 0.5f * v[i] + (v[i] > 0.f ? a.p0 * v[i] * v[i] : a.p1 * (__expf(fminf(v[i], 0.f)) - 1.f - v[i]));
  } else if (a.epi == LIN_TANH_F && feature >= a.n_wide) {
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = tanhf(v[i]);
  }
  if (feature < a.n_wide) *reinterpret_cast<four*>(reinterpret_cast<T*>(a.out_t) + (size_t)row * a.ld_t + feature) = to_four<T>(v);
  else *reinterpret_cast<f32x4*>(a.out_f + (size_t)row * a.ld_f + feature - a.n_wide) = v;
}
template <typename T>
DEV void store_glu(const LinArgs& a, int row, int feature, const f32x4& g, const f32x4& u) {
  typedef typename Frag<T>::four four;
  f32x4 v;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = glu(g[i], u[i], a.p0, a.p1, a.p2);
  *reinterpret_cast<four*>(reinterpret_cast<T*>(a.out_t) + (size_t)row * a.ld_t + feature) = to_four<T>(v);
}

// Workgroups go round robin over the 8 XCDs, each with an L2 of its own: XCD x takes the x-th eighth of the tiles, in order, so that the
// tiles of one weight tile (and then its neighbours) meet in one L2.
DEV int xcd_range(int b, int n) {
  const int x = b & 7, base = n >> 3, extra = n & 7;
  return x * base + min(x, extra) + (b >> 3);
}
// k tiles per part: even, so that a part is whole steps of the prompt kernels
__host__ DEV int part_tiles(int kt, int parts) { return parts > 1 ? ((kt / 2 + parts - 1) / parts) * 2 : kt; }
__host__ DEV int part_tiles(const LinArgs& a) { return part_tiles(a.kt, a.parts); }
// the operand a product's features from `feature` on read
template <typename T>
DEV const T* operand(const LinArgs& a, int feature) {
  const T* p = reinterpret_cast<const T*>(a.a_t);
  return a.a_seg ? p + (size_t)min(feature / a.a_seg, a.a_ops - 1) * a.a_stride : p;
}

// ---- prompts -------------------------------------------------------------------------------------
// grid.x: row tiles of 128 (experts: entries of the tile table), grid.y: feature tiles of 128.
// rows: a gather table (slot -> row) or nullptr; out rows are row0 + local row.
template <typename T>
DEV void lin_body(const LinArgs& a, const int* gather, int row0, int n_rows, int f0, int k0, int k1, char* lds) {
  typedef typename Frag<T>::type frag;
  constexpr int AB = 64 * (int)sizeof(frag);  // bytes of an A fragment
  constexpr int STAGE = 16 * 1024 + 16 * AB;  // 8 row tiles x 2 k tiles of each operand
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wm = wave & 1, wn = wave >> 1;
  const int rt0 = f0 >> 4;
  // this wave's share of the staging: weight tiles rt0 + 2 * wave + {0, 1}, row groups 2 * wave + {0, 1}, both k tiles of a step
  const char* src_w[2];
  const T* src_a[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int t = 2 * wave + i;
    const int rt = min(rt0 + t, a.rt - 1);  // (tiles past the end: any valid one, never stored)
    src_w[i] = reinterpret_cast<const char*>(a.w) + (size_t)rt * a.kt * 1024 + lane * 16;
    int r = min(t * 16 + (sizeof(T) == 2 ? block_row(lane) : lane & 15), n_rows - 1);
    r = gather ? gather[row0 + r] : row0 + r;
    src_a[i] = operand<T>(a, f0) + (size_t)r * a.lda + (sizeof(T) == 2 ? block_group(lane) : lane >> 4) * 8;
  }
  auto stage = [&](int kt, char* buf) {
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const int slot = (2 * wave + i) * 2 + kk;
        __builtin_amdgcn_global_load_lds((gptr)(src_w[i] + (size_t)(kt + kk) * 1024), (lptr)(buf + slot * 1024), 16, 0, 0);
        const char* s = reinterpret_cast<const char*>(src_a[i] + (size_t)(kt + kk) * 32);
#pragma unroll
        for (int h = 0; h < (int)sizeof(T) / 2; ++h)
          __builtin_amdgcn_global_load_lds((gptr)(s + h * 16), (lptr)(buf + 16 * 1024 + slot * AB + h * 1024), 16, 0, 0);
      }
  };
  auto read_a = [&](const char* buf, int slot) {
    frag f;
    if constexpr (sizeof(T) == 2) {
      f = *reinterpret_cast<const frag*>(buf + 16 * 1024 + slot * AB + block_place(lane) * 16);
    } else {
      const f32x4 lo = *reinterpret_cast<const f32x4*>(buf + 16 * 1024 + slot * AB + lane * 16);
      const f32x4 hi = *reinterpret_cast<const f32x4*>(buf + 16 * 1024 + slot * AB + 1024 + lane * 16);
      f = __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7);
    }
    return f;
  };
  f32x4 acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  stage(k0, lds + ((k0 >> 1) & 1) * STAGE);
  for (int kt = k0; kt < k1; kt += 2) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this wave's loads into LDS; the barrier makes it everybody's
    __syncthreads();
    char* cur = lds + ((kt >> 1) & 1) * STAGE;
    if (kt + 2 < k1) stage(kt + 2, lds + (((kt >> 1) & 1) ^ 1) * STAGE);
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8 w[4];
      frag x[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) w[i] = *reinterpret_cast<const bf16x8*>(cur + ((wm * 4 + i) * 2 + kk) * 1024 + lane * 16);
#pragma unroll
      for (int j = 0; j < 4; ++j) x[j] = read_a(cur, (wn * 4 + j) * 2 + kk);
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][j] = mma(w[i], x[j], acc[i][j]);
    }
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = wn * 64 + j * 16 + (lane & 15);
    if (r >= n_rows) continue;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int rt = rt0 + wm * 4 + i;
      if (rt >= a.rt) continue;
      if (a.epi == LIN_GLU) {
        if (!(i & 1)) store_glu<T>(a, row0 + r, (rt >> 1) * 16 + (lane >> 4) * 4, acc[i][j], acc[i | 1][j]);
      } else {
        store_plain<T>(a, row0 + r, rt * 16 + (lane >> 4) * 4, acc[i][j]);
      }
    }
  }
}
template <typename T>
__global__ __launch_bounds__(256) void lin_kernel(LinArgs a, const int row_tiles, const int tiles) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int b = xcd_range(blockIdx.x, tiles), row0 = b % row_tiles * 128, per = part_tiles(a), k0 = blockIdx.y * per;
  a.out_f += blockIdx.y * a.part_stride;
  lin_body<T>(a, nullptr, row0, min(128, a.rows - row0), b / row_tiles * 128, k0, min(a.kt, k0 + per), lds);
}

// 256 features x 256 rows per workgroup: 8 waves of 128 x 64; twice the matrix work per byte staged.  A ring of RING stages of one k tile
// (32 KiB): while a tile is multiplied the next one's operands are read into the other set of registers, and RING - 1 more are on their way.
enum { RING = 4 };
__global__ __launch_bounds__(512) __attribute__((amdgpu_waves_per_eu(2, 2))) void lin_big_kernel(LinArgs a, const int row_tiles, const int tiles) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  constexpr int STAGE = 32 * 1024;
  const int b = xcd_range(blockIdx.x, tiles), row0 = b % row_tiles * 256, f0 = b / row_tiles * 256, per = part_tiles(a), k0 = blockIdx.y * per, n = min(a.kt - k0, per);
  a.out_f += blockIdx.y * a.part_stride;
  const int n_rows = min(256, a.rows - row0);
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wm = wave & 1, wn = wave >> 1, rt0 = f0 >> 4;
  const char *src_w[2], *src_a[2];  // this wave's share of a stage: weight tiles and row groups 2 * wave + {0, 1}
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int t = 2 * wave + i;
    src_w[i] = reinterpret_cast<const char*>(a.w) + ((size_t)min(rt0 + t, a.rt - 1) * a.kt + k0) * 1024 + lane * 16;
    src_a[i] = reinterpret_cast<const char*>(operand<bf16>(a, f0) + (size_t)(row0 + min(t * 16 + block_row(lane), n_rows - 1)) * a.lda + (size_t)k0 * 32 + block_group(lane) * 8);
  }
  auto stage = [&](int kt, char* buf) {  // (past the end: the last tile again, never read)
    kt = min(kt, n - 1);
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int slot = 2 * wave + i;
      __builtin_amdgcn_global_load_lds((gptr)(src_w[i] + (size_t)kt * 1024), (lptr)(buf + slot * 1024), 16, 0, 0);
      __builtin_amdgcn_global_load_lds((gptr)(src_a[i] + (size_t)kt * 64), (lptr)(buf + 16 * 1024 + slot * 1024), 16, 0, 0);
    }
  };
  f32x4 acc[8][4];
#pragma unroll
  for (int i = 0; i < 8; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
  struct Operands {
    bf16x8 w[8], x[4];
  };
  auto read = [&](const char* buf, Operands& o) {
#pragma unroll
    for (int j = 0; j < 4; ++j) o.x[j] = *reinterpret_cast<const bf16x8*>(buf + 16 * 1024 + (wn * 4 + j) * 1024 + block_place(lane) * 16);
#pragma unroll
    for (int i = 0; i < 8; ++i) o.w[i] = *reinterpret_cast<const bf16x8*>(buf + (wm * 8 + i) * 1024 + lane * 16);
  };
  int cur = 0;
  auto step = [&](int kt, const Operands& now, Operands& next) {
    // tile kt + 1 is here when at most the loads of RING - 2 tiles are outstanding; behind the barrier everybody's are, and everybody holds
    // tile kt in registers, so that its buffer takes tile kt + RING
    asm volatile("s_waitcnt vmcnt(%0)" ::"n"(4 * (RING - 2)) : "memory");
    lds_barrier();
    stage(kt + RING, lds + cur * STAGE);
    cur = cur + 1 == RING ? 0 : cur + 1;
    read(lds + cur * STAGE, next);
#pragma unroll
    for (int i = 0; i < 8; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[i][j] = mma(now.w[i], now.x[j], acc[i][j]);
#pragma unroll
    for (int i = 0; i < 12; ++i) {  // one LDS read, then matrix work that does not wait for it
      __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
      __builtin_amdgcn_sched_group_barrier(0x008, 2, 0);
    }
    __builtin_amdgcn_sched_group_barrier(0x008, 8, 0);
  };
  Operands p, q;
#pragma unroll
  for (int i = 0; i < RING; ++i) stage(i, lds + i * STAGE);
  asm volatile("s_waitcnt vmcnt(%0)" ::"n"(4 * (RING - 1)) : "memory");
  lds_barrier();
  read(lds, p);
  for (int kt = 0; kt < n; kt += 2) {  // (n is even)
    step(kt, p, q);
    step(kt + 1, q, p);
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = wn * 64 + j * 16 + (lane & 15);
    if (r >= n_rows) continue;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int rt = rt0 + wm * 8 + i;
      if (rt < a.rt) store_plain<bf16>(a, row0 + r, rt * 16 + (lane >> 4) * 4, acc[i][j]);
    }
  }
}

static LinArgs expert_lin(const MoeArgs& m, bool down) {  // the parts of an expert product that do not depend on the expert
  LinArgs a{};
  a.a_t = down ? m.hidden_t : m.h_t;
  a.lda = down ? m.hidden_ld : m.width_ld;
  a.epi = down ? LIN_STORE : LIN_GLU;
  a.out_t = down ? m.y_t : m.hidden_t;
  a.ld_t = down ? m.y_ld : m.hidden_ld;
  a.n_wide = 0x7fffffff;
  a.p1 = m.alpha;
  a.p2 = m.offset;
  return a;
}
DEV void set_expert(LinArgs& a, const MoeArgs& m, const ExpertMat& e, int expert) {
  const bool sh = expert == m.experts;
  a.w = sh ? e.shared : e.w + (size_t)expert * e.stride;
  a.kt = sh ? e.shared_kt : e.kt;
  a.rt = sh ? e.shared_rt : e.rt;
  a.p0 = sh ? m.shared_limit : m.limit;
}
template <typename T>
__global__ __launch_bounds__(256) void expert_kernel(LinArgs a, const MoeArgs m, const int down) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  if ((int)blockIdx.x >= *m.n_tiles) return;
  const int expert = m.tiles[4 * blockIdx.x], s0 = m.tiles[4 * blockIdx.x + 1], n = m.tiles[4 * blockIdx.x + 2];
  set_expert(a, m, down ? m.down : m.up, expert);
  if ((int)blockIdx.y * 8 >= a.rt) return;
  lin_body<T>(a, down ? nullptr : m.slot_row, s0, n, blockIdx.y * 128, 0, a.kt, lds);
}

// ---- up to 16 rows -------------------------------------------------------------------------------
// One workgroup = 16 features (32 with a gate / up pair): wave w takes k tiles w, w + 4, ...; partial sums meet in LDS.
// row_of: A row of this lane's column; keep: out row or -1.
template <typename T, int NR>
DEV void few_body(const LinArgs& a, int rt0, int k_first, int k_end, int a_row, int out_row, float* lds) {
  typedef typename Frag<T>::type frag;
  constexpr int U = NR == 1 && sizeof(T) == 2 ? 8 : 4;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const bf16x8* w0 = reinterpret_cast<const bf16x8*>(a.w) + (size_t)rt0 * a.kt * 64 + lane;
  const T* x0 = operand<T>(a, rt0 * 16) + (size_t)a_row * a.lda + (lane >> 4) * 8;
  f32x4 acc[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = k_first + wave; k0 < k_end; k0 += 4 * U) {
    bf16x8 w[U][NR];
    frag x[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = min(k0 + 4 * u, k_end - 1);
#pragma unroll
      for (int i = 0; i < NR; ++i) w[u][i] = w0[((size_t)i * a.kt + k) * 64];
      x[u] = *reinterpret_cast<const frag*>(x0 + (size_t)k * 32);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (k0 + 4 * u < k_end)
#pragma unroll
        for (int i = 0; i < NR; ++i) acc[i] = mma(w[u][i], x[u], acc[i]);
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) *reinterpret_cast<f32x4*>(lds + ((wave * NR + i) * 64 + lane) * 4) = acc[i];
  __syncthreads();
  if (wave != 0) return;
#pragma unroll
  for (int i = 0; i < NR; ++i) {
#pragma unroll
    for (int v = 1; v < 4; ++v) acc[i] += *reinterpret_cast<const f32x4*>(lds + ((v * NR + i) * 64 + lane) * 4);
  }
  if (out_row < 0) return;
  if constexpr (NR == 2) store_glu<T>(a, out_row, (rt0 >> 1) * 16 + (lane >> 4) * 4, acc[0], acc[1]);
  else store_plain<T>(a, out_row, rt0 * 16 + (lane >> 4) * 4, acc[0]);
}

struct FewArgs {
  LinArgs t[4];
  int wg_end[4];   // workgroups of products 0 .. i
  int n;
  int expert_wgs;  // in front of them: expert blocks
  int tiles_per_expert;
  int down;
  LinArgs e;
  MoeArgs m;
};
template <typename T>
__global__ __launch_bounds__(256) void few_kernel(const FewArgs f) {
  __shared__ __attribute__((aligned(16))) float lds[4 * 2 * 64 * 4];
  const int c = threadIdx.x & 15;
  int b = blockIdx.x;
  if (b < f.expert_wgs) {
    const int i = b / f.tiles_per_expert, tile = b % f.tiles_per_expert;
    if (i >= *f.m.n_active) return;
    const int expert = f.m.active[i];
    LinArgs a = f.e;
    set_expert(a, f.m, f.down ? f.m.down : f.m.up, expert);
    const int nr = f.down ? 1 : 2;
    if (tile * nr >= a.rt) return;
    const int row = min(c, f.m.rows - 1);
    const int slot = f.m.active_slot[i * 16 + row];
    const int pos = row * (f.m.top + f.m.shared) + max(slot, 0);
    const int out = c < f.m.rows && slot >= 0 ? pos : -1;
    if (f.down) few_body<T, 1>(a, tile, 0, a.kt, pos, out, lds);
    else few_body<T, 2>(a, tile * 2, 0, a.kt, row, out, lds);
    return;
  }
  b -= f.expert_wgs;
  int i = 0;
  while (i + 1 < f.n && b >= f.wg_end[i]) ++i;
  LinArgs a = f.t[i];
  if (i > 0) b -= f.wg_end[i - 1];
  const int row = min(c, a.rows - 1), part = b / a.rt, per = part_tiles(a);
  a.out_f += part * a.part_stride;
  few_body<T, 1>(a, b % a.rt, part * per, min(a.kt, part * per + per), a.row_seq ? a.seqs[a.row_seq[row]].row0 : row, c < a.rows ? c : -1, lds);
}

// ---- launches ------------------------------------------------------------------------------------
static int lin_lds(bool f32) { return 2 * (16 * 1024 + 16 * 64 * (f32 ? 32 : 16)); }
static int check_lin(const LinArgs& a, const char* what) {
  if (!a.w || !a.a_t || a.rows < 1 || a.kt < 2 || (a.kt & 1) || a.rt < 1 || a.lda < a.kt * 32) DSK_FAIL(DSK_ERR_INVALID, "%s: rows %d kt %d rt %d lda %d", what, a.rows, a.kt, a.rt, a.lda);
  if (a.parts > 1 && (a.n_wide || a.epi != LIN_STORE || part_tiles(a) * (a.parts - 1) >= a.kt)) DSK_FAIL(DSK_ERR_INVALID, "%s: %d parts of %d", what, a.parts, a.kt);
  if (a.a_seg < 0 || (a.a_seg & 15) || (a.a_seg && a.a_ops < 1)) DSK_FAIL(DSK_ERR_INVALID, "%s: %d features per operand", what, a.a_seg);
  return DSK_OK;
}
template <typename K>
static int allow_lds(K k, int bytes) {
  HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, bytes));
  return DSK_OK;
}
// Microseconds a prompt product takes on 256 compute units, by measurement: two workgroups of 128 x 128 on one work 1.3 us on a step of 64
// columns (one alone 1.05), one of 256 x 256 takes 1.84 us and starts and ends slower; a part more writes and reads its sums.
static double lin_cost(int rows, int rt, int kt, int parts, bool big) {
  const double k = part_tiles(kt, parts) / 2, sums = (parts - 1) * 3.2e-5 * rows * rt;
  if (big) return cdiv(cdiv(rows, 256) * cdiv(rt, 16) * parts, 256) * (15 + 1.84 * k) + sums;
  const int n = cdiv(rows, 128) * cdiv(rt, 8) * parts;
  return (n <= 256 ? 1.05 * k : cdiv(n, 512) * 1.3 * k) + 5 + sums;
}
static bool lin_big(const LinArgs& a, int parts, bool f32) {
  if (f32 || (a.a_seg & 255)) return false;
  return a.tile ? a.tile == 256 : lin_cost(a.rows, a.rt, a.kt, parts, true) < lin_cost(a.rows, a.rt, a.kt, parts, false);
}
int lin_parts(int rows, int rt, int kt, bool f32, int most) {
  int best = 1;
  double least = 0;
  for (int n = 1; n <= most && (n == 1 || kt / n >= 16); ++n) {
    const double c = std::min(lin_cost(rows, rt, kt, n, false), f32 ? 1e9 : lin_cost(rows, rt, kt, n, true));
    if (n == 1 || c < least) {
      least = c;
      best = n;
    }
  }
  return cdiv(kt, part_tiles(kt, best));  // (no part may be empty)
}
int lin_parts_few(int rt, int kt, int most) {
  const int n = std::max(std::min({1024 / rt, kt / 16, most}), 1);
  return cdiv(kt, part_tiles(kt, n));
}
int launch_lin(hipStream_t st, const LinArgs& a, bool f32) {
  DSK_TRY(check_lin(a, "lin"));
  if ((a.a_seg & 127) || a.row_seq) DSK_FAIL(DSK_ERR_INVALID, "lin: %d features per operand", a.a_seg);
  if (lin_big(a, std::max(a.parts, 1), f32)) {
    const int row_tiles = cdiv(a.rows, 256), tiles = row_tiles * cdiv(a.rt, 16);
    DSK_TRY(allow_lds(lin_big_kernel, RING * 32 * 1024));
    hipLaunchKernelGGL(lin_big_kernel, dim3(tiles, std::max(a.parts, 1)), dim3(512), RING * 32 * 1024, st, a, row_tiles, tiles);
    return DSK_OK;
  }
  const int row_tiles = cdiv(a.rows, 128), tiles = row_tiles * cdiv(a.rt, 8);
  const dim3 grid(tiles, std::max(a.parts, 1));
  const int lds = lin_lds(f32);
  if (f32) {
    DSK_TRY(allow_lds(lin_kernel<float>, lds));
    hipLaunchKernelGGL(lin_kernel<float>, grid, dim3(256), lds, st, a, row_tiles, tiles);
  } else {
    DSK_TRY(allow_lds(lin_kernel<bf16>, lds));
    hipLaunchKernelGGL(lin_kernel<bf16>, grid, dim3(256), lds, st, a, row_tiles, tiles);
  }
  return DSK_OK;
}
int launch_experts(hipStream_t st, const MoeArgs& m, bool down, bool f32) {
  const LinArgs a = expert_lin(m, down);
  const ExpertMat& e = down ? m.down : m.up;
  const dim3 grid(m.max_tiles, cdiv(m.shared ? (e.rt > e.shared_rt ? e.rt : e.shared_rt) : e.rt, 8));
  const int lds = lin_lds(f32);
  if (f32) {
    DSK_TRY(allow_lds(expert_kernel<float>, lds));
    hipLaunchKernelGGL(expert_kernel<float>, grid, dim3(256), lds, st, a, m, (int)down);
  } else {
    DSK_TRY(allow_lds(expert_kernel<bf16>, lds));
    hipLaunchKernelGGL(expert_kernel<bf16>, grid, dim3(256), lds, st, a, m, (int)down);
  }
  return DSK_OK;
}
static int launch_few(hipStream_t st, FewArgs& f, const LinArgs* a, int n, bool f32) {
  if (n > 4) DSK_FAIL(DSK_ERR_INVALID, "lin_few: %d products", n);
  f.n = n;
  int wgs = 0;
  for (int i = 0; i < n; ++i) {
    DSK_TRY(check_lin(a[i], "lin_few"));
    if (a[i].rows > 16) DSK_FAIL(DSK_ERR_INVALID, "lin_few: %d rows", a[i].rows);
    f.t[i] = a[i];
    f.wg_end[i] = wgs += a[i].rt * std::max(a[i].parts, 1);
  }
  const dim3 grid(f.expert_wgs + wgs);
  if (f32) hipLaunchKernelGGL(few_kernel<float>, grid, dim3(256), 0, st, f);
  else hipLaunchKernelGGL(few_kernel<bf16>, grid, dim3(256), 0, st, f);
  return DSK_OK;
}
int launch_lin_few(hipStream_t st, const LinArgs* a, int n, bool f32) {
  FewArgs f{};
  return launch_few(st, f, a, n, f32);
}
int launch_experts_few(hipStream_t st, const MoeArgs& m, bool down, const LinArgs* also, int n_also, bool f32) {
  if (m.rows > 16) DSK_FAIL(DSK_ERR_INVALID, "experts_few: %d rows", m.rows);
  FewArgs f{};
  f.m = m;
  f.down = down;
  f.e = expert_lin(m, down);
  const ExpertMat& e = down ? m.down : m.up;
  const int rt = m.shared ? (e.rt > e.shared_rt ? e.rt : e.shared_rt) : e.rt;
  f.tiles_per_expert = down ? rt : rt / 2;
  f.expert_wgs = m.max_active * f.tiles_per_expert;
  return launch_few(st, f, also, n_also, f32);
}
