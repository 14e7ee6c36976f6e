// kernels_latent.hip -- latent attention of layered models in a sliding window: position i sees j with 0 <= i - j < window.
//
// A token leaves one row: its normed latent c [rank_p] and the rotated key part shared by all heads [rot_p].  A sequence keeps the last
// `window` of them in a ring.
//   latent_prep     norms of the query latent and of c, the angles' cosines and sines, the rotated key part
//   latent_gather   the older rows that a portion of several tokens sees, from the ring, in front of the portion's rows; one matrix product
//                   then expands them all to keys and values per head
//   latent_turn     the rotation of the queries
//   latent_attn     64 queries per workgroup (attn_tile.h): a key is its head's expanded part, then the shared rotated one
//   latent_store    the portion's last rows into the ring (behind the attention's gather)
//   latent_few      single tokens: the query comes carried into the latent space (W_uk^T q), so a score is one product with a ring row and
//                   all heads of a token share the rows: one workgroup per (token, 64 rows), heads as the columns of the MFMA, the rows
//                   staged once in LDS for scores and weighted sums alike
//   latent_values   merges the workgroups' parts of a head and expands the weighted latent to the head's values (W_uv)
#include "attn_tile.h"
#include "layered_kernels.h"

#include <math.h>

#include <algorithm>

static int cdiv(int a, int b) { return (a + b - 1) / b; }
template <typename T>
struct FewKeys {
  enum { N = sizeof(T) == 2 ? 64 : 32 };  // ring rows per workgroup of latent_few
};
int latent_keys(bool f32) { return f32 ? (int)FewKeys<float>::N : (int)FewKeys<bf16>::N; }

// element j of a rotated part [rot_p] whose raw values come from x(j); turn: cosines, then sines
template <typename X>
DEV float turned(X x, const float* turn, int rot_dims, int j) {
  const int half = rot_dims >> 1;
  const float v = x(j);
  if (j >= rot_dims) return v;
  return j < half ? v * turn[j] - x(j + half) * turn[half + j] : v * turn[j - half] + x(j - half) * turn[j];
}

// ---- norms and rotation: one workgroup per row --------------------------------------------------------------
enum { PREP_NT = 512 };
template <typename T>
__global__ __launch_bounds__(PREP_NT) void latent_prep_kernel(const LatentArgs a) {
  constexpr int NT = PREP_NT, U = 4;  // U elements of either latent per thread wait in registers; larger ones are read again
  __shared__ float red[2 * NT / 64];
  const int row = blockIdx.x, tid = threadIdx.x, half = a.rot_dims >> 1, ld = a.rank_p + a.rot_p, cq_k = (a.q_rank + 63) & ~63;
  const SeqDesc s = a.p.seqs[a.p.row_seq[row]];
  const int pos = s.pos0 + row - s.row0;
  const float *q = a.proj_f + (size_t)row * a.ld + a.col_q, *kv = a.proj_f + (size_t)row * a.ld + a.col_kv;
  float xq[U], xk[U], wq[U], wk[U], sq = 0.f, sk = 0.f;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int i = tid + u * NT;
    xq[u] = i < a.q_rank ? q[i] : 0.f;
    wq[u] = i < a.q_rank ? a.q_norm[i] : 0.f;
    xk[u] = i < a.kv_rank ? kv[i] : 0.f;
    wk[u] = i < a.kv_rank ? a.kv_norm[i] : 0.f;
  }
  float* turn = a.turn + (size_t)row * a.rot_dims;
  for (int i = tid; i < half; i += NT) {
    float sn, cs;
    sincosf((float)pos * a.freq[i], &sn, &cs);
    turn[i] = cs;
    turn[half + i] = sn;
  }
#pragma unroll
  for (int u = 0; u < U; ++u) {
    sq += xq[u] * xq[u];
    sk += xk[u] * xk[u];
  }
  for (int i = tid + U * NT; i < a.q_rank; i += NT) sq += q[i] * q[i];
  for (int i = tid + U * NT; i < a.kv_rank; i += NT) sk += kv[i] * kv[i];
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((tid & 63) == 0) {
    red[tid >> 6] = sq;
    red[NT / 64 + (tid >> 6)] = sk;
  }
  __syncthreads();  // (the cosines and sines too: this workgroup's own stores are visible to it behind the barrier)
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) {
    sq += red[i];
    sk += red[NT / 64 + i];
  }
  const float rq = 1.f / sqrtf(sq / a.q_rank + a.eps), rk = 1.f / sqrtf(sk / a.kv_rank + a.eps);
  T* cq = reinterpret_cast<T*>(a.cq_t) + (size_t)row * a.cq_ld;
  T* lat = s.len == 1 ? reinterpret_cast<T*>(s.state + a.off_c) + (size_t)(pos % a.window) * ld : reinterpret_cast<T*>(a.lat_t) + (size_t)(s.key0 + s.hist + row - s.row0) * ld;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int i = tid + u * NT;
    if (i < cq_k) cq[i] = (T)(xq[u] * rq * wq[u]);
    if (i < a.rank_p) lat[i] = (T)(xk[u] * rk * wk[u]);
  }
  for (int i = tid + U * NT; i < cq_k; i += NT) cq[i] = (T)(i < a.q_rank ? q[i] * rq * a.q_norm[i] : 0.f);
  for (int i = tid + U * NT; i < a.rank_p; i += NT) lat[i] = (T)(i < a.kv_rank ? kv[i] * rk * a.kv_norm[i] : 0.f);
  for (int j = tid; j < a.rot_p; j += NT) lat[a.rank_p + j] = (T)(j < a.rot_dim ? turned([&](int i) { return kv[a.kv_rank + i]; }, turn, a.rot_dims, j) : 0.f);
}

// ---- rows between ring and key workspace -----------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void latent_gather_kernel(const LatentArgs a) {
  typedef typename Frag<T>::type frag;
  const SeqDesc s = a.p.seqs[blockIdx.y];
  const int ld = a.rank_p + a.rot_p, wave = threadIdx.x >> 6;
  if (s.len == 1) return;
  for (int u = 0; u < 4; ++u) {
    const int i = blockIdx.x * 16 + wave * 4 + u, pos = s.pos0 - s.hist + i;
    if (i >= s.hist || pos <= s.pos0 - a.window) continue;  // (`hist` goes by the widest window of the model)
    const T* src = reinterpret_cast<const T*>(s.state + a.off_c) + (size_t)(pos % a.window) * ld;
    T* dst = reinterpret_cast<T*>(a.lat_t) + (size_t)(s.key0 + i) * ld;
    for (int e = (threadIdx.x & 63) * 8; e < ld; e += 512) *reinterpret_cast<frag*>(dst + e) = *reinterpret_cast<const frag*>(src + e);
  }
}
template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(const LatentArgs a) {
  typedef typename Frag<T>::type frag;
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6), ld = a.rank_p + a.rot_p;
  if (row >= a.p.rows) return;
  const SeqDesc s = a.p.seqs[a.p.row_seq[row]];
  const int t = row - s.row0;
  if (s.len == 1 || t < s.len - a.window) return;
  const T* src = reinterpret_cast<const T*>(a.lat_t) + (size_t)(s.key0 + s.hist + t) * ld;
  T* dst = reinterpret_cast<T*>(s.state + a.off_c) + (size_t)((s.pos0 + t) % a.window) * ld;
  for (int e = (threadIdx.x & 63) * 8; e < ld; e += 512) *reinterpret_cast<frag*>(dst + e) = *reinterpret_cast<const frag*>(src + e);
}

// ---- rotation of the queries, in place (portions of several tokens; latent_few rotates its own) -----------------------
template <typename T>
__global__ __launch_bounds__(256) void latent_turn_kernel(const LatentArgs a) {
  const int row = blockIdx.x, half = a.rot_dims >> 1, hd = a.dim_p + a.rot_p;
  if (a.p.seqs[a.p.row_seq[row]].len == 1) return;
  const float* turn = a.turn + (size_t)row * a.rot_dims;
  T* q = reinterpret_cast<T*>(a.q_t) + (size_t)row * a.q_ld + a.dim_p;
#pragma unroll 4
  for (int i = threadIdx.x; i < a.heads * half; i += 256) {
    const int j = i % half;
    T* p = q + (size_t)(i / half) * hd + j;
    const float u = (float)p[0], v = (float)p[half], c = turn[j], s = turn[half + j];
    p[0] = (T)(u * c - v * s);
    p[half] = (T)(v * c + u * s);
  }
}

// ---- portions of several tokens --------------------------------------------------------------------------------------
template <typename T>
struct LatentKeys {
  typedef typename Frag<T>::type frag;
  typedef typename Frag<T>::four four;
  const LatentArgs& a;
  const SeqDesc& s;
  int h;
  DEV int first(int pos) const { return max(0, pos - a.window + 1); }
  DEV size_t key_row(int pos) const { return (size_t)(s.key0 + s.hist + pos - s.pos0); }
  DEV frag q(int row, int gr) const {
    return *reinterpret_cast<const frag*>(reinterpret_cast<const T*>(a.q_t) + (size_t)(s.row0 + row) * a.q_ld + (size_t)h * (a.dim_p + a.rot_p) + gr * 8);
  }
  DEV frag k(int pos, int gr) const {
    const size_t r = key_row(pos);
    const T* p = gr * 8 < a.dim_p ? reinterpret_cast<const T*>(a.kv_t) + r * a.kv_ld + (size_t)h * a.dim_p
                                  : reinterpret_cast<const T*>(a.lat_t) + r * (a.rank_p + a.rot_p) + a.rank_p - a.dim_p;
    return *reinterpret_cast<const frag*>(p + gr * 8);
  }
  DEV four v(int pos, int c) const {
    return *reinterpret_cast<const four*>(reinterpret_cast<const T*>(a.kv_t) + key_row(pos) * a.kv_ld + (size_t)a.heads * a.dim_p + (size_t)h * a.vdim_p + c);
  }
};
template <typename T, int KT, int VTL>
ATTN_KERNEL(T) void latent_attn_kernel(const LatentArgs a) {
  const int h = blockIdx.y, tile = gridDim.x - 1 - blockIdx.x;  // (a sequence's last tiles have the most keys: they start first)
  const SeqDesc s = a.p.seqs[a.p.qtile[2 * tile]];
  if (s.len == 1) return;
  attn_tile<T, KT, VTL>(LatentKeys<T>{a, s, h}, s, a.p.qtile[2 * tile + 1], (a.dim_p + a.rot_p) >> 5, a.vdim_p >> 4, a.vdim, a.scale,
                        reinterpret_cast<T*>(a.out_t) + h * a.vdim, a.out_ld);
}

// ---- single tokens -----------------------------------------------------------------------------------------------------
enum { FEW_NT = 512, FEW_NW = 8 };
template <typename T>
static size_t few_lds(int rank_p, int rot_p) {
  const size_t n = FewKeys<T>::N;
  return n * (rank_p + rot_p + 16 / sizeof(T)) * sizeof(T) + 16 * (size_t)(rot_p + 8) * sizeof(T) + FEW_NW * 64 * 16 + 16 * (n + 8) * sizeof(T);
}
template <typename T>
__global__ __launch_bounds__(FEW_NT) void latent_few_kernel(const LatentArgs a) {
  typedef typename Frag<T>::type frag;
  constexpr int N = FewKeys<T>::N, KTILES = N / 16, PARTS = FEW_NW / KTILES, LP = N + 8;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), g = lane >> 4, c16 = lane & 15;
  const int i = blockIdx.y, split = blockIdx.x;
  const SeqDesc s = a.p.seqs[a.p.single[a.first + i]];
  const int pos = s.pos0, seen = min(pos + 1, a.window), k0 = split * N, n = min(N, seen - k0);
  if (n <= 0) return;
  const int ld = a.rank_p + a.rot_p, LD = ld + 16 / (int)sizeof(T), LQ = a.rot_p + 8;
  T* lat = reinterpret_cast<T*>(lds);                     // [N][LD]
  T* qr = lat + (size_t)N * LD;                           // [16][LQ] rotated parts of a head tile's queries
  f32x4* red = reinterpret_cast<f32x4*>(qr + 16 * LQ);    // [PARTS][KTILES][64]
  T* pw = reinterpret_cast<T*>(red + FEW_NW * 64);        // [16][LP] weights
  const T* ring = reinterpret_cast<const T*>(s.state + a.off_c);
  const int ng = ld >> 3, first = pos - seen + 1 + k0;
  // the query operands of a wave's part, ahead of everything else (the first ones; larger latents read the rest as they go)
  constexpr int QA = sizeof(T) == 2 ? 8 : 4;
  const int kt16 = wave % KTILES, part = wave / KTILES, kts = a.rank_p >> 5;
  frag qf[QA];
  auto query = [&](int h0) { return reinterpret_cast<const T*>(a.qa_t) + ((size_t)i * a.heads + min(h0 + c16, a.heads - 1)) * a.rank_p + g * 8; };
  auto ahead = [&](int h0) {
#pragma unroll
    for (int u = 0; u < QA; ++u) qf[u] = *reinterpret_cast<const frag*>(query(h0) + min(part + u * PARTS, kts - 1) * 32);
  };
  ahead(0);
  constexpr int IN_FLIGHT = sizeof(T) == 2 ? 12 : 6;
  for (int u0 = tid; u0 < N * ng; u0 += FEW_NT * IN_FLIGHT) {
    frag f[IN_FLIGHT];
#pragma unroll
    for (int j = 0; j < IN_FLIGHT; ++j) {
      const int u = u0 + j * FEW_NT, key = u / ng, gr = u % ng;
      f[j] = frag{};
      if (key < n) f[j] = *reinterpret_cast<const frag*>(ring + (size_t)((first + key) % a.window) * ld + gr * 8);
    }
#pragma unroll
    for (int j = 0; j < IN_FLIGHT; ++j) {
      const int u = u0 + j * FEW_NT;
      if (u < N * ng) *reinterpret_cast<frag*>(lat + (size_t)(u / ng) * LD + u % ng * 8) = f[j];
    }
  }
  const float* turn = a.turn + (size_t)s.row0 * a.rot_dims;
  const int hd = a.dim_p + a.rot_p;
  for (int h0 = 0; h0 < a.heads; h0 += 16) {
    for (int u = tid; u < 16 * a.rot_p; u += FEW_NT) {
      const int hh = u / a.rot_p, j = u % a.rot_p;
      const T* q = reinterpret_cast<const T*>(a.q_t) + (size_t)s.row0 * a.q_ld + (size_t)min(h0 + hh, a.heads - 1) * hd + a.dim_p;
      qr[hh * LQ + j] = (T)(j < a.rot_dim ? turned([&](int e) { return (float)q[e]; }, turn, a.rot_dims, j) : 0.f);
    }
    __syncthreads();
    {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
      auto score = [&](int kt, const frag& q) { acc = mma(*reinterpret_cast<const frag*>(lat + (size_t)(kt16 * 16 + c16) * LD + kt * 32 + g * 8), q, acc); };
#pragma unroll
      for (int u = 0; u < QA; ++u)
        if (part + u * PARTS < kts) score(part + u * PARTS, qf[u]);
      for (int kt = part + QA * PARTS; kt < kts; kt += PARTS) score(kt, *reinterpret_cast<const frag*>(query(h0) + kt * 32));
      for (int kt = part; kt < a.rot_p >> 5; kt += PARTS) score(kts + kt, *reinterpret_cast<const frag*>(qr + c16 * LQ + kt * 32 + g * 8));
      if (h0 + 16 < a.heads) ahead(h0 + 16);
      red[(part * KTILES + kt16) * 64 + lane] = acc;
    }
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 16 / FEW_NW; ++u) {  // a wave's heads of the tile: lane = key
      const int hh = wave * (16 / FEW_NW) + u;
      float sc = -INFINITY;
      if (lane < n) {
        sc = 0.f;
#pragma unroll
        for (int p = 0; p < PARTS; ++p) sc += red[(p * KTILES + (lane >> 4)) * 64 + ((lane >> 2) & 3) * 16 + hh][lane & 3];
        sc *= a.scale;
      }
      float m = sc;
#pragma unroll
      for (int off = 32; off >= 1; off >>= 1) m = fmaxf(m, __shfl_xor(m, off));
      const float w = expf(sc - m), l = wave_sum(w);
      if (lane < N) pw[hh * LP + lane] = (T)w;
      if (lane == 0 && h0 + hh < a.heads) {
        float* ml = a.part_ml + (((size_t)i * a.heads + h0 + hh) * a.splits + split) * 2;
        ml[0] = m;
        ml[1] = l;
      }
    }
    __syncthreads();
    frag p[N / 32];
#pragma unroll
    for (int ks = 0; ks < N / 32; ++ks) p[ks] = *reinterpret_cast<const frag*>(pw + c16 * LP + ks * 32 + g * 8);
    float* out = a.part + (((size_t)i * a.heads + min(h0 + c16, a.heads - 1)) * a.splits + split) * a.rank_p;
    for (int ct = wave; ct < a.rank_p >> 4; ct += FEW_NW) {
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < N / 32; ++ks) {
        frag v;
#pragma unroll
        for (int e = 0; e < 8; ++e) v[e] = lat[(size_t)(ks * 32 + g * 8 + e) * LD + ct * 16 + c16];
        acc = mma(v, p[ks], acc);
      }
      if (h0 + c16 < a.heads) *reinterpret_cast<f32x4*>(out + ct * 16 + g * 4) = acc;
    }
  }
}
// one workgroup per (head, 64 values, token)
template <typename T>
__global__ __launch_bounds__(256) void latent_values_kernel(const LatentArgs a) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = blockIdx.x, v0 = blockIdx.y * 64, i = blockIdx.z;
  const SeqDesc s = a.p.seqs[a.p.single[a.first + i]];
  const int n = (min(s.pos0 + 1, a.window) + FewKeys<T>::N - 1) / FewKeys<T>::N;
  float* c = reinterpret_cast<float*>(lds);  // [rank_p] merged latent
  float* w = c + a.rank_p;                   // [splits] weights of the parts
  float* red = w + (a.splits + 3) / 4 * 4;   // [4][64]
  const int r = v0 + lane, R = a.up_row + h * a.vdim_p + min(r, a.vdim_p - 1), ng = a.rank_p >> 3;
  const bf16* W = reinterpret_cast<const bf16*>(a.up_w) + (size_t)(R >> 4) * a.up_kt * 512 + (R & 15) * 8;
  constexpr int AHEAD = 16;                  // this thread's first weights, requested before anything else
  bf16x8 x[AHEAD];
#pragma unroll
  for (int u = 0; u < AHEAD; ++u) {
    const int gr = min(wave + 4 * u, ng - 1);
    x[u] = *reinterpret_cast<const bf16x8*>(W + (size_t)(gr >> 2) * 512 + (gr & 3) * 128);
  }
  const float* ml = a.part_ml + ((size_t)i * a.heads + h) * a.splits * 2;
  float m = -INFINITY, l = 0.f;              // (every wave for itself)
  for (int k = lane; k < n; k += 64) m = fmaxf(m, ml[2 * k]);
#pragma unroll
  for (int off = 32; off >= 1; off >>= 1) m = fmaxf(m, __shfl_xor(m, off));
  for (int k = lane; k < n; k += 64) {
    const float e = expf(ml[2 * k] - m);
    l += e * ml[2 * k + 1];
    if (wave == 0) w[k] = e;
  }
  l = wave_sum(l);
  __syncthreads();
  const float* part = a.part + ((size_t)i * a.heads + h) * a.splits * a.rank_p;
  for (int e = tid * 4; e < a.rank_p; e += 1024) {
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < n; k0 += 8) {
      f32x4 v[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) v[u] = *reinterpret_cast<const f32x4*>(part + (size_t)min(k0 + u, n - 1) * a.rank_p + e);
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (k0 + u < n) o += w[k0 + u] * v[u];
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) c[e + j] = (float)(T)(o[j] / l);
  }
  __syncthreads();
  float z = 0.f;
#pragma unroll
  for (int u = 0; u < AHEAD; ++u) {
    const int gr = wave + 4 * u;
    if (gr < ng)
#pragma unroll
      for (int e = 0; e < 8; ++e) z += (float)x[u][e] * c[gr * 8 + e];
  }
  for (int gr = wave + 4 * AHEAD; gr < ng; gr += 4) {
    const bf16x8 y = *reinterpret_cast<const bf16x8*>(W + (size_t)(gr >> 2) * 512 + (gr & 3) * 128);
#pragma unroll
    for (int e = 0; e < 8; ++e) z += (float)y[e] * c[gr * 8 + e];
  }
  red[wave * 64 + lane] = z;
  __syncthreads();
  if (wave == 0 && r < a.vdim) reinterpret_cast<T*>(a.out_t)[(size_t)s.row0 * a.out_ld + h * a.vdim + r] = (T)((red[lane] + red[64 + lane]) + (red[128 + lane] + red[192 + lane]));
}

// ---- launches --------------------------------------------------------------------------------------------------------------
static int check_latent(const LatentArgs& a, bool f32) {
  const size_t lds = f32 ? few_lds<float>(a.rank_p, a.rot_p) : few_lds<bf16>(a.rank_p, a.rot_p);
  if (a.dim_p + a.rot_p > 256 || a.vdim_p > 256 || lds > 160 * 1024 || (a.rot_dims & 1) || a.rot_dims > a.rot_dim)
    DSK_FAIL(DSK_ERR_UNSUPPORTED, "latent attention: key size %d + %d, value size %d (max 256), latent size %d", a.dim, a.rot_dim, a.vdim, a.kv_rank);
  return DSK_OK;
}
int launch_latent_prep(hipStream_t st, const LatentArgs& a, bool f32) {
  DSK_TRY(check_latent(a, f32));
  if (f32) hipLaunchKernelGGL(latent_prep_kernel<float>, dim3(a.p.rows), dim3(PREP_NT), 0, st, a);
  else hipLaunchKernelGGL(latent_prep_kernel<bf16>, dim3(a.p.rows), dim3(PREP_NT), 0, st, a);
  return DSK_OK;
}
int launch_latent_gather(hipStream_t st, const LatentArgs& a, bool f32) {
  if (a.p.max_hist < 1) return DSK_OK;
  const dim3 grid(cdiv(a.p.max_hist, 16), a.p.n_seqs);
  if (f32) hipLaunchKernelGGL(latent_gather_kernel<float>, grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL(latent_gather_kernel<bf16>, grid, dim3(256), 0, st, a);
  return DSK_OK;
}
int launch_latent_turn(hipStream_t st, const LatentArgs& a, bool f32) {
  if (a.rot_dims < 2) return DSK_OK;
  if (f32) hipLaunchKernelGGL(latent_turn_kernel<float>, dim3(a.p.rows), dim3(256), 0, st, a);
  else hipLaunchKernelGGL(latent_turn_kernel<bf16>, dim3(a.p.rows), dim3(256), 0, st, a);
  return DSK_OK;
}
int launch_latent_store(hipStream_t st, const LatentArgs& a, bool f32) {
  const dim3 grid(cdiv(a.p.rows, 4));
  if (f32) hipLaunchKernelGGL(latent_store_kernel<float>, grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL(latent_store_kernel<bf16>, grid, dim3(256), 0, st, a);
  return DSK_OK;
}
template <typename T>
static int attn_t(hipStream_t st, const LatentArgs& a) {
  return attn_sizes((a.dim_p + a.rot_p) >> 5, a.vdim_p >> 4, [&](auto kt, auto vt) -> int {
    constexpr int KT = decltype(kt)::value, VTL = decltype(vt)::value, lds = attn_tile_lds<T, KT, VTL>();
    auto k = latent_attn_kernel<T, KT, VTL>;
    HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    hipLaunchKernelGGL(k, dim3(a.p.n_qtiles, a.heads), dim3(256), lds, st, a);
    return (int)DSK_OK;
  }, "latent attention");
}
int launch_latent_attn(hipStream_t st, const LatentArgs& a, bool f32) {
  DSK_TRY(check_latent(a, f32));
  return f32 ? attn_t<float>(st, a) : attn_t<bf16>(st, a);
}
template <typename T>
static int few_t(hipStream_t st, const LatentArgs& a) {
  const size_t lds = few_lds<T>(a.rank_p, a.rot_p), lds_v = ((size_t)a.rank_p + (a.splits + 3) / 4 * 4 + 256) * 4;
  HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(latent_few_kernel<T>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  hipLaunchKernelGGL(latent_few_kernel<T>, dim3(a.splits, a.n), dim3(FEW_NT), lds, st, a);
  HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(latent_values_kernel<T>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds_v));
  hipLaunchKernelGGL(latent_values_kernel<T>, dim3(a.heads, cdiv(a.vdim, 64), a.n), dim3(256), lds_v, st, a);
  return DSK_OK;
}
int launch_latent_few(hipStream_t st, const LatentArgs& a, bool f32) {
  DSK_TRY(check_latent(a, f32));
  if (a.n < 1 || a.n > 16 || a.splits < 1) DSK_FAIL(DSK_ERR_INVALID, "latent_few: %d tokens", a.n);
  return f32 ? few_t<float>(st, a) : few_t<bf16>(st, a);
}
