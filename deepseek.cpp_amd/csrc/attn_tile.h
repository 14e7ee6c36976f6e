// attn_tile.h -- softmax attention of 64 queries of one head over a contiguous range of keys, for the attention kernels of layered models.
//
// 4 waves of 16 queries, key tiles of 64 through LDS, online softmax in 32-bit.  Scores come out of the MFMA with the query in the lane
// and four keys in the registers, which is the operand order of the second product when v's key order is permuted alike: the weights
// never leave their registers.  The next tile's keys and values travel to registers while the current one is worked off.
#pragma once
#include "layered_kernels.h"
#include "seq_device.h"

#include <math.h>

// LDS: a tile of 64 keys as fragments [4 x 16 keys][dim / 32][64 lanes][8], then v transposed [vdim][64 keys + pad]
enum { ATTN_KEYS = 64 };
template <typename T>
struct VT {
  enum { LD = ATTN_KEYS + (sizeof(T) == 2 ? 8 : 4) };  // elements per row of the transposed v tile
};
template <typename T>
static size_t attn_tile_lds(int dim_p, int vdim_p) {
  return ((size_t)ATTN_KEYS * dim_p + (size_t)vdim_p * VT<T>::LD) * sizeof(T);
}
// weights x values for 32 keys of a tile: keys 4 g + i of the first 16 and of the second 16 (g = lane / 16)
DEV f32x4 mma_pv(const bf16* v, const f32x4& p0, const f32x4& p1, const f32x4& acc) {
  typedef bf16 b4 __attribute__((ext_vector_type(4)));
  const b4 v0 = *reinterpret_cast<const b4*>(v), v1 = *reinterpret_cast<const b4*>(v + 16);
  const bf16x8 vv = __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7);
  const bf16x8 pp = __builtin_shufflevector(to_four<bf16>(p0), to_four<bf16>(p1), 0, 1, 2, 3, 4, 5, 6, 7);
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, pp, acc, 0, 0, 0);
}
DEV f32x4 mma_pv(const float* v, const f32x4& p0, const f32x4& p1, f32x4 acc) {
  const f32x4 v0 = *reinterpret_cast<const f32x4*>(v), v1 = *reinterpret_cast<const f32x4*>(v + 16);
#pragma unroll
  for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(v0[i], p0[i], acc, 0, 0, 0);
#pragma unroll
  for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(v1[i], p1[i], acc, 0, 0, 0);
  return acc;
}
// One workgroup of 256: rows [q0, q0 + 64) of portion s.  Keys: where queries, keys and values come from (groups of 8 elements, 4 value
// channels) and the first position a position sees; it sees itself and everything in between.  kts = padded key size / 32 <= KT,
// vts = padded value size / 16 <= VTL.
template <typename T, int KT, int VTL, typename Keys>
DEV void attn_tile(const Keys& src, const SeqDesc& sq, int q0, int kts, int vts, int vdim, float scale, T* out, int out_ld) {
  typedef typename Frag<T>::type frag;
  typedef typename Frag<T>::four four;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  constexpr int NS = ATTN_KEYS / 16, KI = KT * NS / 4, VI = VTL * NS / 16;  // a wave's share of a tile: KI fragments of keys, VI blocks of values
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int nq = min(64, sq.len - q0);
  T* kf = reinterpret_cast<T*>(lds);                     // fragments of the key tile
  T* vt = kf + (size_t)NS * kts * 512;                   // transposed values
  const int my_q = min(q0 + wave * 16 + (lane & 15), sq.len - 1);
  const int my_pos = sq.pos0 + my_q, my_first = src.first(my_pos);
  frag q[KT];
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
    if (kt < kts) q[kt] = src.q(my_q, kt * 4 + (lane >> 4));
  f32x4 o[VTL];
#pragma unroll
  for (int i = 0; i < VTL; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  const int first = src.first(sq.pos0 + q0), last = sq.pos0 + q0 + nq - 1;
  // A wave loads whole fragments of keys (16 keys x 32 elements: 64 bytes a row, lane-linear in LDS), and blocks of 32 keys x 32 value
  // channels (8 lanes a row; the transposed writes of 8 rows meet every LDS bank once).
  const int kr = lane & 15, kg = lane >> 4, vc = (lane & 7) * 4, vk = (lane >> 3) * 4;
  frag rk[KI];
  four rv[VI][4];
  auto fetch = [&](int j0) {  // keys past the tile's last position repeat it (masked below)
#pragma unroll
    for (int u = 0; u < KI; ++u) {
      const int id = wave + 4 * u, kt = id / NS;
      if (kt < kts) rk[u] = src.k(min(j0 + id % NS * 16 + kr, last), kt * 4 + kg);
    }
#pragma unroll
    for (int u = 0; u < VI; ++u) {
      const int id = wave + 4 * u, c = id / (NS / 2) * 32 + vc;
      if (c < vts * 16)
#pragma unroll
        for (int k = 0; k < 4; ++k) rv[u][k] = src.v(min(j0 + id % (NS / 2) * 32 + vk + k, last), c);
    }
  };
  fetch(first);
  for (int j0 = first; j0 <= last; j0 += ATTN_KEYS) {
    __syncthreads();
#pragma unroll
    for (int u = 0; u < KI; ++u) {
      const int id = wave + 4 * u, kt = id / NS;
      if (kt < kts) *reinterpret_cast<frag*>(kf + (((size_t)(id % NS) * kts + kt) * 64 + lane) * 8) = rk[u];
    }
#pragma unroll
    for (int u = 0; u < VI; ++u) {
      const int id = wave + 4 * u, c = id / (NS / 2) * 32 + vc;
      if (c < vts * 16)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          *reinterpret_cast<four*>(vt + (size_t)(c + e) * VT<T>::LD + id % (NS / 2) * 32 + vk) = four{rv[u][0][e], rv[u][1][e], rv[u][2][e], rv[u][3][e]};
    }
    __syncthreads();
    if (j0 + ATTN_KEYS <= last) fetch(j0 + ATTN_KEYS);
    if (wave * 16 >= nq || j0 > sq.pos0 + q0 + min(wave * 16 + 15, nq - 1)) continue;  // (barriers above: every wave passes them)
    f32x4 s[NS];
#pragma unroll
    for (int t = 0; t < NS; ++t) {
      s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
        if (kt < kts) s[t] = mma(*reinterpret_cast<const frag*>(kf + (((size_t)t * kts + kt) * 64 + lane) * 8), q[kt], s[t]);
    }
    float mx = m;
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int pos = j0 + t * 16 + (lane >> 4) * 4 + i;
        s[t][i] = pos <= my_pos && pos >= my_first ? s[t][i] * scale : -INFINITY;
        mx = fmaxf(mx, s[t][i]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float ref = mx == -INFINITY ? 0.f : mx;  // nothing visible yet: every weight below is exp(-inf) = 0
    const float old = expf(m - ref);
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[t][i] = expf(s[t][i] - ref);
        sum += s[t][i];
      }
    sum += __shfl_xor(sum, 16);
    sum += __shfl_xor(sum, 32);
    l = l * old + sum;
    m = mx;
#pragma unroll
    for (int i = 0; i < VTL; ++i)
      if (i < vts) {
        o[i] *= old;
#pragma unroll
        for (int t = 0; t < NS; t += 2) o[i] = mma_pv(vt + (size_t)(i * 16 + (lane & 15)) * VT<T>::LD + t * 16 + (lane >> 4) * 4, s[t], s[t + 1], o[i]);
      }
  }
  const int qi = wave * 16 + (lane & 15);
  if (qi >= nq) return;
  out += (size_t)(sq.row0 + q0 + qi) * out_ld;
#pragma unroll
  for (int i = 0; i < VTL; ++i)
    if (i < vts)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int c = i * 16 + (lane >> 4) * 4 + e;
        if (c < vdim) out[c] = (T)(o[i][e] / l);
      }
}
