// kernels_chunk_scan.hip -- the recurrences of layered models over chunks of 16 tokens, as 32-bit matrix products.
//
// Inside a chunk that starts from the state S0 [dim][vdim], with G_t the product of the decays of its tokens up to t (per key channel)
// and all ratios of such products taken as products of the decays in between (they are at most 1: nothing overflows):
//   delta rule   u_t = beta_t (v_t - (k_t G_t)^T S0 - sum_{s<t} A_ts u_s),    A_ts = sum_d k_t k_s G_t / G_s
//                o_t = (q_t G_t)^T S0 + sum_{s<=t} B_ts u_s,                  B_ts = sum_d q_t k_s G_t / G_s
//                S  <- G_16 S0 + sum_s (k_s G_16 / G_s) u_s^T
//   mLSTM        the same without A (u = v); the decay is one number per token, exp(f + m_before - m), and k_s carries exp(i_s - m_s).
//                A column of ones behind v makes the normaliser n one more column of S.
//   wkv          the same without A, read before the write: o_t = (q_t G_(t-1))^T S0 + sum_{s<=t} B_ts v_s with B_ts = sum_d q_t k_s
//                G_(t-1) / G_s below the diagonal, and the bonus on it: B_tt = sum_d q_t u k_t
// *_prepare: everything that does not depend on S0, for all chunks at once - the operands with decays multiplied in, B, and
// T = (I + diag(beta) A)^-1 diag(beta), so that U = T (V - Kg S0).  chunk_scan: one workgroup per (16 columns, head, sequence)
// goes through the chunks; its 4 waves share the key channels.  S stays in MFMA accumulators: their layout (column = lane % 16, rows
// 4 (lane / 16) + i) is an operand layout of v_mfma_f32_16x16x4_f32 when step i stands for the k values {4 g + i}.
#include "layered_kernels.h"
#include "seq_device.h"

#include <math.h>

static int cdiv(int a, int b) { return (a + b - 1) / b; }
enum { CH = RECUR_CHUNK };

struct Ops {  // one chunk's operands of one head
  float *kg, *qg, *ke, *gend, *t, *b;
};
DEV Ops ops_at(float* base, size_t chunk, int heads, int h, int dim) {
  const int dp = (dim + 15) / 16 * 16;
  Ops o;
  o.kg = base + (chunk * heads + h) * (49 * (size_t)dp + 512);
  o.qg = o.kg + 16 * dp;
  o.ke = o.qg + 16 * dp;
  o.gend = o.ke + 16 * dp;
  o.t = o.gend + dp;
  o.b = o.t + 256;
  return o;
}

// ---- delta rule: operands -----------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void delta_prepare_kernel(const DeltaArgs a, float* __restrict__ base) {
  extern __shared__ float lds[];
  const int tid = threadIdx.x, h = blockIdx.y, dim = a.dim, dp = (dim + 15) / 16 * 16;
  float *sk = lds, *sq = sk + 16 * dp, *sg = sq + 16 * dp, *sA = sg + 16 * dp, *sb = sA + 16 * 17;
  const SeqDesc s = a.p.seqs[a.p.chunk[2 * blockIdx.x]];
  const int t0 = a.p.chunk[2 * blockIdx.x + 1], n = min((int)CH, s.len - t0);
  const int kv = h / (a.heads / a.kv_heads), nq = a.kv_heads * dim;
  const size_t row0 = (size_t)s.row0 + t0;
  for (int i = tid; i < 16 * dp; i += 256) {  // rows past the end: no key, no query, no decay
    const int t = i / dp, d = i % dp;
    const bool in = t < n && d < dim;
    sk[i] = in ? a.k[(row0 + t) * nq + (size_t)kv * dim + d] : 0.f;
    sq[i] = in ? a.q[(row0 + t) * nq + (size_t)kv * dim + d] : 0.f;
    sg[i] = in ? (a.head_decay ? a.g[(row0 + t) * a.heads + h] : a.g[(row0 + t) * a.heads * dim + (size_t)h * dim + d]) : 1.f;
  }
  if (tid < 16) sb[tid] = tid < n ? a.beta[(row0 + tid) * a.heads + h] : 0.f;
  __syncthreads();
  const Ops o = ops_at(base, blockIdx.x, a.heads, h, dim);
  for (int d = tid; d < dp; d += 256) {
    float G = 1.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      G *= sg[t * dp + d];
      o.kg[t * dp + d] = sk[t * dp + d] * G;
      o.qg[t * dp + d] = sq[t * dp + d] * G;
    }
    o.gend[d] = G;
    float E = 1.f, e[16];
#pragma unroll
    for (int t = 15; t >= 0; --t) {
      e[t] = sk[t * dp + d] * E;
      E *= sg[t * dp + d];
    }
#pragma unroll
    for (int t = 0; t < 16; t += 4) *reinterpret_cast<f32x4*>(o.ke + (size_t)d * 16 + t) = f32x4{e[t], e[t + 1], e[t + 2], e[t + 3]};
  }
  // A and B: thread -> (token s, every 16th channel), all later tokens t in registers
  const int sx = tid >> 4, dg = tid & 15;
  float aA[16], aB[16];
#pragma unroll
  for (int t = 0; t < 16; ++t) aA[t] = aB[t] = 0.f;
  for (int d = dg; d < dp; d += 16) {
    float w = 0.f;
    const float ks = sk[sx * dp + d];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      w = t == sx ? ks : w * sg[t * dp + d];
      aA[t] += sk[t * dp + d] * w;
      aB[t] += sq[t * dp + d] * w;
    }
  }
#pragma unroll
  for (int t = 0; t < 16; ++t) {
    const float A = row_sum(aA[t]), B = row_sum(aB[t]);
    if (dg == t) {
      sA[t * 17 + sx] = A;
      o.b[t * 16 + sx] = sx <= t ? B : 0.f;
    }
  }
  __syncthreads();
  if (tid < 16) {  // column tid of T, by forward substitution
    float x[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float r = 0.f;
#pragma unroll
      for (int u = 0; u < t; ++u) r += sA[t * 17 + u] * x[u];
      x[t] = sb[t] * ((t == tid ? 1.f : 0.f) - r);
      o.t[t * 16 + tid] = x[t];
    }
  }
}

// ---- mLSTM: running maximum, operands --------------------------------------------------------------------------
// m_t = max(f_t + m_(t-1), i_t) composes: (F, I) then (f, i) = (F + f, max(I + f, i)); one wave per (head, sequence), 64 tokens a turn
__global__ __launch_bounds__(64) void mlstm_gates_kernel(const MlstmArgs a, const ChunkScan c) {
  const int lane = threadIdx.x, h = blockIdx.x;
  const SeqDesc s = a.p.seqs[blockIdx.y];
  float* M = reinterpret_cast<float*>(s.state + a.off_m) + h;
  float m = s.pos0 > 0 ? M[s.flip * a.heads] : 0.f;
  for (int t0 = 0; t0 < s.len; t0 += 64) {
    const int t = t0 + lane;
    const bool in = t < s.len;
    const size_t row = (size_t)s.row0 + (in ? t : 0);
    const float* G = a.gate_f + row * a.ld_gate;
    const float i = in ? a.gate_cap * tanhf((G[a.col_i + h] + a.b_i[h]) / a.gate_cap) : -INFINITY;
    const float f = in ? logsigmoid_f(a.gate_cap * tanhf((G[a.col_f + h] + a.b_f[h]) / a.gate_cap)) : 0.f;
    float F = f, I = i;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const float pF = __shfl_up(F, off), pI = __shfl_up(I, off);
      if (lane >= off) {
        I = fmaxf(pI + F, I);
        F += pF;
      }
    }
    const float mt = fmaxf(F + m, I);
    float before = __shfl_up(mt, 1);
    if (lane == 0) before = m;
    if (in) {
      c.keep[row * a.heads + h] = expf(fminf(f + before - mt, 0.f));
      c.add[row * a.heads + h] = expf(fminf(i - mt, 0.f));
      c.floor[row * a.heads + h] = expf(-mt);
    }
    m = __shfl(mt, 63);  // (lanes past the end carry it on)
  }
  if (lane == 0) M[(s.flip ^ 1) * a.heads] = m;
}
template <typename T>
__global__ __launch_bounds__(256) void mlstm_prepare_kernel(const MlstmArgs a, const ChunkScan c) {
  extern __shared__ float lds[];
  const int tid = threadIdx.x, h = blockIdx.y, dim = a.dim, dp = (dim + 15) / 16 * 16;
  float *sk = lds, *sq = sk + 16 * dp, *keep = sq + 16 * dp, *add = keep + 16;
  const SeqDesc s = a.p.seqs[a.p.chunk[2 * blockIdx.x]];
  const int t0 = a.p.chunk[2 * blockIdx.x + 1], n = min((int)CH, s.len - t0);
  const size_t row0 = (size_t)s.row0 + t0;
  for (int i = tid; i < 16 * dp; i += 256) {
    const int t = i / dp, d = i % dp;
    const bool in = t < n && d < dim;
    const T* P = reinterpret_cast<const T*>(a.proj_t) + (row0 + (in ? t : 0)) * a.ld + h * dim + (in ? d : 0);
    sk[i] = in ? (float)P[a.col_k] : 0.f;
    sq[i] = in ? (float)P[a.col_q] * a.q_scale : 0.f;
  }
  if (tid < 16) {
    keep[tid] = tid < n ? c.keep[(row0 + tid) * a.heads + h] : 1.f;
    add[tid] = tid < n ? c.add[(row0 + tid) * a.heads + h] : 0.f;
  }
  __syncthreads();
  const Ops o = ops_at(c.ops, blockIdx.x, a.heads, h, dim);
  for (int d = tid; d < dp; d += 256) {
    float G = 1.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      G *= keep[t];
      o.qg[t * dp + d] = sq[t * dp + d] * G;
    }
    o.gend[d] = G;
    float E = 1.f, e[16];
#pragma unroll
    for (int t = 15; t >= 0; --t) {
      e[t] = sk[t * dp + d] * add[t] * E;
      E *= keep[t];
    }
#pragma unroll
    for (int t = 0; t < 16; t += 4) *reinterpret_cast<f32x4*>(o.ke + (size_t)d * 16 + t) = f32x4{e[t], e[t + 1], e[t + 2], e[t + 3]};
  }
  const int sx = tid >> 4, dg = tid & 15;
  float acc[16];
#pragma unroll
  for (int t = 0; t < 16; ++t) acc[t] = 0.f;
  for (int d = dg; d < dp; d += 16) {
    const float ks = sk[sx * dp + d];
#pragma unroll
    for (int t = 0; t < 16; ++t) acc[t] += sq[t * dp + d] * ks;
  }
  float w = 0.f;
#pragma unroll
  for (int t = 0; t < 16; ++t) {
    w = t == sx ? add[sx] : w * keep[t];
    const float B = row_sum(acc[t]) * w;
    if (dg == t) o.b[t * 16 + sx] = sx <= t ? B : 0.f;
  }
}

// ---- wkv: operands ------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void wkv_prepare_kernel(const WkvArgs a, float* __restrict__ base) {
  extern __shared__ float lds[];
  const int tid = threadIdx.x, h = blockIdx.y, dim = a.dim, dp = (dim + 15) / 16 * 16;
  float *sk = lds, *sq = sk + 16 * dp, *sg = sq + 16 * dp, *su = sg + 16 * dp;
  const SeqDesc s = a.p.seqs[a.p.chunk[2 * blockIdx.x]];
  const int t0 = a.p.chunk[2 * blockIdx.x + 1], n = min((int)CH, s.len - t0);
  const size_t row0 = (size_t)s.row0 + t0;
  for (int i = tid; i < 16 * dp; i += 256) {  // rows past the end: no key, no query, no decay
    const int t = i / dp, d = i % dp;
    const bool in = t < n && d < dim;
    const size_t row = row0 + (in ? t : 0);
    const int c = h * dim + (in ? d : 0);
    const T* P = reinterpret_cast<const T*>(a.proj_t) + row * a.ld + c;
    sk[i] = in ? (float)P[a.col_k] : 0.f;
    sq[i] = in ? (float)P[a.col_r] : 0.f;
    sg[i] = in ? expf(-expf(a.low_f[row * a.ld_low + c] + a.w0[c])) : 1.f;
  }
  for (int d = tid; d < dp; d += 256) su[d] = d < dim ? a.u[h * dim + d] : 0.f;
  __syncthreads();
  const Ops o = ops_at(base, blockIdx.x, a.heads, h, dim);
  for (int d = tid; d < dp; d += 256) {
    float G = 1.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      o.qg[t * dp + d] = sq[t * dp + d] * G;
      G *= sg[t * dp + d];
    }
    o.gend[d] = G;
    float E = 1.f, e[16];
#pragma unroll
    for (int t = 15; t >= 0; --t) {
      e[t] = sk[t * dp + d] * E;
      E *= sg[t * dp + d];
    }
#pragma unroll
    for (int t = 0; t < 16; t += 4) *reinterpret_cast<f32x4*>(o.ke + (size_t)d * 16 + t) = f32x4{e[t], e[t + 1], e[t + 2], e[t + 3]};
  }
  const int sx = tid >> 4, dg = tid & 15;
  float acc[16];
#pragma unroll
  for (int t = 0; t < 16; ++t) acc[t] = 0.f;
  for (int d = dg; d < dp; d += 16) {
    float w = 0.f;
    const float ks = sk[sx * dp + d];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      acc[t] += sq[t * dp + d] * (t == sx ? ks * su[d] : w);
      w = t == sx ? ks : w * sg[t * dp + d];
    }
  }
#pragma unroll
  for (int t = 0; t < 16; ++t) {
    const float B = row_sum(acc[t]);
    if (dg == t) o.b[t * 16 + sx] = sx <= t ? B : 0.f;
  }
}

// ---- the chunks of a sequence, one after the other -------------------------------------------------------------
struct ScanArgs {
  PassDesc p;
  int heads, dim, vdim;
  float* ops;
  const void* v;       // delta: floats [rows][heads * vdim]; mLSTM: proj_t + col_v
  int ld_v;
  float* o;            // [rows][heads][cols]
  size_t off_s, off_n;
};
enum { SCAN_DELTA, SCAN_MLSTM, SCAN_WKV };
template <typename T, int KIND, int NTL>
__global__ __launch_bounds__(256) void chunk_scan_kernel(const ScanArgs a) {
  constexpr bool DELTA = KIND == SCAN_DELTA, NORM = KIND == SCAN_MLSTM;
  __shared__ __attribute__((aligned(16))) f32x4 ex[2][4][2][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, c16 = lane & 15;
  const int h = blockIdx.y, dp = (a.dim + 15) / 16 * 16, tiles = dp >> 4;
  const int cols = NORM ? a.vdim + 1 : a.vdim;
  const int col = blockIdx.x * 16 + c16;
  const bool live = col < cols, norm = NORM && col == a.vdim;
  const SeqDesc s = a.p.seqs[blockIdx.z];
  float* S0 = reinterpret_cast<float*>(s.state + a.off_s) + (size_t)h * a.dim * a.vdim;
  float* N0 = !NORM ? nullptr : reinterpret_cast<float*>(s.state + a.off_n) + (size_t)h * a.dim;
  const size_t nn = (size_t)a.heads * a.dim;
  f32x4 S[NTL];
#pragma unroll
  for (int i = 0; i < NTL; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int k = (wave + 4 * i) * 16 + g * 4 + e;
      S[i][e] = s.pos0 > 0 && live && k < a.dim ? (norm ? N0[s.flip * nn + k] : S0[(size_t)k * a.vdim + col]) : 0.f;
    }
  // Requested without a branch and untouched until they are used, so that the waits count exactly: rows past the end repeat the last
  // one (their columns of T, B and Ke are zero), columns past the last one compute something nobody stores.
  struct Operands {
    f32x4 kg[NTL], qg[NTL], ke[NTL], ge[NTL], t, b;
    T v[4];
  };
  const int vcol = min(col, a.vdim - 1);
  const int nc = (s.len + CH - 1) / CH;
  auto load = [&](int c, Operands& x) {
    c = min(c, nc - 1);
    const Ops o = ops_at(a.ops, (size_t)s.chunk0 + c, a.heads, h, a.dim);
#pragma unroll
    for (int i = 0; i < NTL; ++i) {
      const int tile = min(wave + 4 * i, tiles - 1);
      if (DELTA) x.kg[i] = *reinterpret_cast<const f32x4*>(o.kg + c16 * dp + tile * 16 + g * 4);
      x.qg[i] = *reinterpret_cast<const f32x4*>(o.qg + c16 * dp + tile * 16 + g * 4);
      x.ke[i] = *reinterpret_cast<const f32x4*>(o.ke + (size_t)(tile * 16 + c16) * 16 + g * 4);
      x.ge[i] = *reinterpret_cast<const f32x4*>(o.gend + tile * 16 + g * 4);
    }
    if (DELTA) x.t = *reinterpret_cast<const f32x4*>(o.t + c16 * 16 + g * 4);
    x.b = *reinterpret_cast<const f32x4*>(o.b + c16 * 16 + g * 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const size_t row = (size_t)s.row0 + min(c * CH + g * 4 + e, s.len - 1);
      x.v[e] = reinterpret_cast<const T*>(a.v)[row * a.ld_v + (size_t)h * a.vdim + vcol];
    }
  };
  auto step = [&](int c, const Operands& x, Operands& fill) {  // fill: the operands of chunk c + 2
    load(c + 2, fill);
    f32x4 W = {0.f, 0.f, 0.f, 0.f}, X = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NTL; ++i)
      if (wave + 4 * i < tiles)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          if (DELTA) W = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kg[i][e], S[i][e], W, 0, 0, 0);
          X = __builtin_amdgcn_mfma_f32_16x16x4f32(x.qg[i][e], S[i][e], X, 0, 0, 0);
        }
    if (DELTA) ex[c & 1][wave][0][lane] = W;
    ex[c & 1][wave][1][lane] = X;
    lds_barrier();  // (the operands of the next chunks stay in flight)
    f32x4 U;
#pragma unroll
    for (int e = 0; e < 4; ++e) U[e] = norm ? 1.f : (float)x.v[e];
    if (DELTA) {
      W = (ex[c & 1][0][0][lane] + ex[c & 1][1][0][lane]) + (ex[c & 1][2][0][lane] + ex[c & 1][3][0][lane]);
      const f32x4 r = U - W;
      U = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int e = 0; e < 4; ++e) U = __builtin_amdgcn_mfma_f32_16x16x4f32(x.t[e], r[e], U, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < NTL; ++i)
      if (wave + 4 * i < tiles) {
        S[i] *= x.ge[i];
#pragma unroll
        for (int e = 0; e < 4; ++e) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.ke[i][e], U[e], S[i], 0, 0, 0);
      }
    if (wave == (c & 3)) {  // the waves take turns with the outputs
      f32x4 O = (ex[c & 1][0][1][lane] + ex[c & 1][1][1][lane]) + (ex[c & 1][2][1][lane] + ex[c & 1][3][1][lane]);
#pragma unroll
      for (int e = 0; e < 4; ++e) O = __builtin_amdgcn_mfma_f32_16x16x4f32(x.b[e], U[e], O, 0, 0, 0);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = c * CH + g * 4 + e;
        if (t < s.len && live) a.o[((size_t)(s.row0 + t) * a.heads + h) * cols + col] = O[e];
      }
    }
  };
  Operands x, y, z;
  load(0, x);
  load(1, y);
  for (int c = 0; c < nc; c += 3) {
    step(c, x, z);
    if (c + 1 < nc) step(c + 1, y, x);
    if (c + 2 < nc) step(c + 2, z, y);
  }
#pragma unroll
  for (int i = 0; i < NTL; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int k = (wave + 4 * i) * 16 + g * 4 + e;
      if (!live || k >= a.dim) continue;
      if (norm) N0[(s.flip ^ 1) * nn + k] = S[i][e];
      else S0[(size_t)k * a.vdim + col] = S[i][e];
    }
}

// ---- launches ------------------------------------------------------------------------------------------------------
template <typename T, int KIND>
static int scan_t(hipStream_t st, const ScanArgs& a) {
  if (a.dim < 1 || a.dim > RECUR_MAX_DIM) DSK_FAIL(DSK_ERR_UNSUPPORTED, "recurrence: key size %d (max %d)", a.dim, (int)RECUR_MAX_DIM);
  const dim3 grid(cdiv(KIND == SCAN_MLSTM ? a.vdim + 1 : a.vdim, 16), a.heads, a.p.n_seqs);
  if (a.dim <= 64) hipLaunchKernelGGL((chunk_scan_kernel<T, KIND, 1>), grid, dim3(256), 0, st, a);
  else if (a.dim <= 128) hipLaunchKernelGGL((chunk_scan_kernel<T, KIND, 2>), grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL((chunk_scan_kernel<T, KIND, 4>), grid, dim3(256), 0, st, a);
  return DSK_OK;
}
int launch_delta_chunks(hipStream_t st, const DeltaArgs& a, const ChunkScan& c) {
  const int dp = (a.dim + 15) / 16 * 16;
  const size_t lds = ((size_t)48 * dp + 16 * 17 + 16) * 4;
  HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(delta_prepare_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  hipLaunchKernelGGL(delta_prepare_kernel, dim3(a.p.n_chunks, a.heads), dim3(256), lds, st, a, c.ops);
  return scan_t<float, SCAN_DELTA>(st, ScanArgs{a.p, a.heads, a.dim, a.vdim, c.ops, a.v, a.heads * a.vdim, a.o, a.off_s, 0});
}
template <typename T>
static int mlstm_t(hipStream_t st, const MlstmArgs& a, const ChunkScan& c) {
  const int dp = (a.dim + 15) / 16 * 16;
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3(a.heads, a.p.n_seqs), dim3(64), 0, st, a, c);
  hipLaunchKernelGGL(mlstm_prepare_kernel<T>, dim3(a.p.n_chunks, a.heads), dim3(256), ((size_t)32 * dp + 32) * 4, st, a, c);
  return scan_t<T, SCAN_MLSTM>(st, ScanArgs{a.p, a.heads, a.dim, a.vdim, c.ops, reinterpret_cast<const T*>(a.proj_t) + a.col_v, a.ld, a.o, a.off_s, a.off_n});
}
int launch_mlstm_chunks(hipStream_t st, const MlstmArgs& a, const ChunkScan& c, bool f32) { return f32 ? mlstm_t<float>(st, a, c) : mlstm_t<bf16>(st, a, c); }
template <typename T>
static int wkv_t(hipStream_t st, const WkvArgs& a, const ChunkScan& c) {
  if (a.dim > RECUR_MAX_DIM) DSK_FAIL(DSK_ERR_UNSUPPORTED, "wkv: key size %d (max %d)", a.dim, (int)RECUR_MAX_DIM);
  const int dp = (a.dim + 15) / 16 * 16;
  hipLaunchKernelGGL(wkv_prepare_kernel<T>, dim3(a.p.n_chunks, a.heads), dim3(256), (size_t)49 * dp * 4, st, a, c.ops);
  return scan_t<T, SCAN_WKV>(st, ScanArgs{a.p, a.heads, a.dim, a.dim, c.ops, reinterpret_cast<const T*>(a.proj_t) + a.col_v, a.ld, a.o, a.off_s, 0});
}
int launch_wkv_chunks(hipStream_t st, const WkvArgs& a, const ChunkScan& c, bool f32) { return f32 ? wkv_t<float>(st, a, c) : wkv_t<bf16>(st, a, c); }
