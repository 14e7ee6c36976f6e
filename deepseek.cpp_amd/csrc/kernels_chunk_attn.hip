// kernels_chunk_attn.hip -- chunked softmax attention of layered models: a position sees the positions of its own chunk up to itself.
// Chunks count from position 0 of the sequence, so a sequence keeps at most one chunk of keys and values: row (position % chunk).
//
//   chunk_prep    rotary positions (interleaved pairs), RMS norm of q and k per head, copies of v; padded to 32 per head
//   chunk_attn    64 queries per workgroup (attn_tile.h)
//   chunk_store   the rows of the sequence's last chunk into its cache (behind the attention, which reads the older ones)
#include "attn_tile.h"
#include "layered_kernels.h"

#include <math.h>

static int cdiv(int a, int b) { return (a + b - 1) / b; }

// ---- rotation, norm, padding: one wave per head ---------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void chunk_prep_kernel(const ChunkAttnArgs a) {
  const int row = blockIdx.x, lane = threadIdx.x & 63;
  const SeqDesc sq = a.p.seqs[a.p.row_seq[row]];
  const float pos = (float)(sq.pos0 + row - sq.row0);
  const T* P = reinterpret_cast<const T*>(a.proj_t) + (size_t)row * a.ld;
  const int n_heads = a.heads + 2 * a.kv_heads;
  for (int hd = blockIdx.y * 4 + (threadIdx.x >> 6); hd < n_heads; hd += gridDim.y * 4) {
    if (hd >= a.heads + a.kv_heads) {
      const int g = hd - a.heads - a.kv_heads;
      T* dst = reinterpret_cast<T*>(a.v_t) + ((size_t)row * a.kv_heads + g) * a.vdim_p;
      for (int i = lane; i < a.vdim_p; i += 64) dst[i] = i < a.vdim ? P[a.col_v + g * a.vdim + i] : (T)0.f;
      continue;
    }
    const bool is_q = hd < a.heads;
    const T* src = P + (is_q ? a.col_q + hd * a.dim : a.col_k + (hd - a.heads) * a.dim);
    T* dst = is_q ? reinterpret_cast<T*>(a.q_t) + ((size_t)row * a.heads + hd) * a.dim_p
                  : reinterpret_cast<T*>(a.k_t) + ((size_t)row * a.kv_heads + hd - a.heads) * a.dim_p;
    float u[2], v[2], ss = 0.f;  // pairs lane and lane + 64 (dim <= 256)
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int pr = lane + 64 * i;
      u[i] = 2 * pr < a.dim ? (float)src[2 * pr] : 0.f;
      v[i] = 2 * pr + 1 < a.dim ? (float)src[2 * pr + 1] : 0.f;
      if (2 * pr < a.rot_dims) {
        float s, c;
        sincosf(pos * a.freq[pr], &s, &c);
        s *= a.rot_amp;
        c *= a.rot_amp;
        const float u1 = u[i] * c - v[i] * s;
        v[i] = v[i] * c + u[i] * s;
        u[i] = u1;
      }
      ss += u[i] * u[i] + v[i] * v[i];
    }
    ss = wave_sum(ss);
    const float r = 1.f / sqrtf(ss / a.dim + a.eps);
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int pr = lane + 64 * i;
      if (2 * pr < a.dim_p) {
        dst[2 * pr] = (T)(u[i] * r);
        dst[2 * pr + 1] = (T)(v[i] * r);
      }
    }
  }
}

// ---- attention -----------------------------------------------------------------------------------------
// keys and values of one head: the portion's from the workspace, older ones of the same chunk from the sequence's cache
template <typename T>
struct ChunkKeys {
  typedef typename Frag<T>::type frag;
  typedef typename Frag<T>::four four;
  const ChunkAttnArgs& a;
  const SeqDesc& s;
  int h, g;
  DEV int first(int pos) const { return pos / a.chunk * a.chunk; }
  DEV frag q(int row, int gr) const { return *reinterpret_cast<const frag*>(reinterpret_cast<const T*>(a.q_t) + ((size_t)(s.row0 + row) * a.heads + h) * a.dim_p + gr * 8); }
  DEV frag k(int pos, int gr) const {
    const T* p = pos >= s.pos0 ? reinterpret_cast<const T*>(a.k_t) + ((size_t)(s.row0 + pos - s.pos0) * a.kv_heads + g) * a.dim_p
                               : reinterpret_cast<const T*>(s.state + a.off_k) + ((size_t)(pos % a.chunk) * a.kv_heads + g) * a.dim_p;
    return *reinterpret_cast<const frag*>(p + gr * 8);
  }
  DEV four v(int pos, int c) const {
    const T* p = pos >= s.pos0 ? reinterpret_cast<const T*>(a.v_t) + ((size_t)(s.row0 + pos - s.pos0) * a.kv_heads + g) * a.vdim_p
                               : reinterpret_cast<const T*>(s.state + a.off_v) + ((size_t)(pos % a.chunk) * a.kv_heads + g) * a.vdim_p;
    return *reinterpret_cast<const four*>(p + c);
  }
};
template <typename T, int KT, int VTL>
ATTN_KERNEL(T) void chunk_attn_kernel(const ChunkAttnArgs a) {
  const int h = blockIdx.y, tile = gridDim.x - 1 - blockIdx.x;  // (a sequence's last tiles have the most keys: they start first)
  const SeqDesc s = a.p.seqs[a.p.qtile[2 * tile]];
  attn_tile<T, KT, VTL>(ChunkKeys<T>{a, s, h, h / (a.heads / a.kv_heads)}, s, a.p.qtile[2 * tile + 1], a.dim_p >> 5, a.vdim_p >> 4, a.vdim, a.scale,
                        reinterpret_cast<T*>(a.out_t) + h * a.vdim, a.out_ld);
}

// ---- cache rows ------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void chunk_store_kernel(const ChunkAttnArgs a) {
  const int row = blockIdx.x;
  const SeqDesc sq = a.p.seqs[a.p.row_seq[row]];
  const int pos = sq.pos0 + row - sq.row0, end = sq.pos0 + sq.len - 1;
  if (pos / a.chunk != end / a.chunk) return;
  const int nk = a.kv_heads * a.dim_p, nv = a.kv_heads * a.vdim_p;
  T* ck = reinterpret_cast<T*>(sq.state + a.off_k) + (size_t)(pos % a.chunk) * nk;
  T* cv = reinterpret_cast<T*>(sq.state + a.off_v) + (size_t)(pos % a.chunk) * nv;
  const T* k = reinterpret_cast<const T*>(a.k_t) + (size_t)row * nk;
  const T* v = reinterpret_cast<const T*>(a.v_t) + (size_t)row * nv;
  for (int i = threadIdx.x; i < nk; i += 256) ck[i] = k[i];
  for (int i = threadIdx.x; i < nv; i += 256) cv[i] = v[i];
}

// ---- launches ---------------------------------------------------------------------------------------------
int launch_chunk_prep(hipStream_t st, const ChunkAttnArgs& a, bool f32) {
  if (a.dim > 256 || a.vdim > 256 || (a.dim & 1)) DSK_FAIL(DSK_ERR_UNSUPPORTED, "chunk attention: key size %d, value size %d (max 256)", a.dim, a.vdim);
  const dim3 grid(a.p.rows, a.p.rows >= 64 ? 1 : cdiv(a.heads + 2 * a.kv_heads, 4));
  if (f32) hipLaunchKernelGGL(chunk_prep_kernel<float>, grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL(chunk_prep_kernel<bf16>, grid, dim3(256), 0, st, a);
  return DSK_OK;
}
template <typename T>
static int attn_t(hipStream_t st, const ChunkAttnArgs& a) {
  return attn_sizes(a.dim_p >> 5, a.vdim_p >> 4, [&](auto kt, auto vt) -> int {
    constexpr int KT = decltype(kt)::value, VTL = decltype(vt)::value, lds = attn_tile_lds<T, KT, VTL>();
    auto k = chunk_attn_kernel<T, KT, VTL>;
    HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, lds));
    hipLaunchKernelGGL(k, dim3(a.p.n_qtiles, a.heads), dim3(256), lds, st, a);
    return (int)DSK_OK;
  }, "chunk attention");
}
int launch_chunk_attn(hipStream_t st, const ChunkAttnArgs& a, bool f32) { return f32 ? attn_t<float>(st, a) : attn_t<bf16>(st, a); }
int launch_chunk_store(hipStream_t st, const ChunkAttnArgs& a, bool f32) {
  if (f32) hipLaunchKernelGGL(chunk_store_kernel<float>, dim3(a.p.rows), dim3(256), 0, st, a);
  else hipLaunchKernelGGL(chunk_store_kernel<bf16>, dim3(a.p.rows), dim3(256), 0, st, a);
  return DSK_OK;
}
