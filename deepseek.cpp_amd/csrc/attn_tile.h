// attn_tile.h -- softmax attention of 64 queries of one head over a contiguous range of keys, for the attention kernels of layered models.
//
// 4 waves of 16 queries, key tiles of 64 through LDS, online softmax in 32-bit.  Scores come out of the MFMA with the query in the lane
// and four keys in the registers, which is the operand order of the second product when v's key order is permuted alike: the weights
// never leave their registers.  The next tile's keys and values travel to registers while the current one is worked off.
#pragma once
#include "layered_kernels.h"
#include "seq_device.h"

#include <math.h>

#include <type_traits>

// LDS: a tile of 64 keys as blocks [4 x 16 keys][dim / 32][64 places][8], then v transposed [vdim][64 keys + pad]
enum { ATTN_KEYS = 64 };
template <typename T>
struct VT {
  enum { LD = ATTN_KEYS + (sizeof(T) == 2 ? 8 : 4) };  // elements per row of the transposed v tile
};
template <typename T, int KT, int VTL>
constexpr int attn_tile_lds() {
  return (ATTN_KEYS * KT * 32 + VTL * 16 * VT<T>::LD) * (int)sizeof(T);
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
// channels) and the first position a position sees; it sees itself and everything in between.  The padded key size is kts k tiles of 32,
// the padded value size vts tiles of 16; KT and VTL, at least as large, are what is worked off, without branches: beyond kts queries are zero
// and the last k tile of the keys comes again, beyond vts the last values come again and nobody stores them.
template <typename T, int KT, int VTL, typename Keys>
DEV void attn_tile(const Keys& src, const SeqDesc& sq, int q0, int kts, int vts, int vdim, float scale, T* out, int out_ld) {
  typedef typename Frag<T>::type frag;
  typedef typename Frag<T>::four four;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  constexpr int NS = ATTN_KEYS / 16, VI = VTL / 4;       // sub-tiles of 16 keys (a wave loads one), blocks of 32 keys x 32 value channels per wave
  static_assert(NS == 4 && VTL % 4 == 0, "a wave per sub-tile of keys, two waves per block of values");
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int nq = min(64, sq.len - q0);
  const float scale2 = scale * 1.44269504f;              // weights as powers of two: one instruction each
  T* kf = reinterpret_cast<T*>(lds);                     // blocks of the key tile
  T* vt = kf + (size_t)NS * KT * 512;                    // transposed values
  const int my_q = min(q0 + wave * 16 + (lane & 15), sq.len - 1);
  const int my_pos = sq.pos0 + my_q, my_first = src.first(my_pos);
  const int first = src.first(sq.pos0 + q0), last = sq.pos0 + q0 + nq - 1;
  // values: 8 lanes to the 64 bytes of a row, 4 rows per lane; the transposed writes meet every LDS bank once
  const int vc = (lane & 7) * 4, vk = (wave & 1) * 32 + (lane >> 3) * 4;
  frag q[KT], rk[KT];
  four rv[VI][4];
#pragma unroll
  for (int kt = 0; kt < KT; ++kt) q[kt] = src.q(my_q, min(kt, kts - 1) * 4 + (lane >> 4));
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
    if (kt >= kts) q[kt] = frag{};
  __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0): inside the loop only the prefetched loads are waited for
  auto fetch = [&](int j0) {  // keys past the tile's last position repeat it (masked below)
    const int pos = min(j0 + wave * 16 + block_row(lane), last);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) rk[kt] = src.k(pos, min(kt, kts - 1) * 4 + block_group(lane));
#pragma unroll
    for (int u = 0; u < VI; ++u)
#pragma unroll
      for (int k = 0; k < 4; ++k) rv[u][k] = src.v(min(j0 + vk + k, last), min((wave >> 1) + 2 * u, (vts >> 1) - 1) * 32 + vc);
  };
  f32x4 o[VTL];
#pragma unroll
  for (int i = 0; i < VTL; ++i) o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  fetch(first);
  for (int j0 = first; j0 <= last; j0 += ATTN_KEYS) {
    __syncthreads();
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) *reinterpret_cast<frag*>(kf + ((size_t)(wave * KT + kt) * 64 + lane) * 8) = rk[kt];
#pragma unroll
    for (int u = 0; u < VI; ++u)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        *reinterpret_cast<four*>(vt + (size_t)(((wave >> 1) + 2 * u) * 32 + vc + e) * VT<T>::LD + vk) = four{rv[u][0][e], rv[u][1][e], rv[u][2][e], rv[u][3][e]};
    __syncthreads();
    if (j0 + ATTN_KEYS <= last) fetch(j0 + ATTN_KEYS);
    if (wave * 16 >= nq || j0 > sq.pos0 + q0 + min(wave * 16 + 15, nq - 1)) continue;  // (barriers above: every wave passes them)
    f32x4 s[NS];
#pragma unroll
    for (int t = 0; t < NS; ++t) {
      s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kt = 0; kt < KT; ++kt) s[t] = mma(*reinterpret_cast<const frag*>(kf + ((size_t)(t * KT + kt) * 64 + block_place(lane)) * 8), q[kt], s[t]);
    }
    float mx = m;
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int pos = j0 + t * 16 + (lane >> 4) * 4 + i;
        s[t][i] = pos <= my_pos && pos >= my_first ? s[t][i] * scale2 : -INFINITY;
        mx = fmaxf(mx, s[t][i]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 16));
    mx = fmaxf(mx, __shfl_xor(mx, 32));
    const float ref = mx == -INFINITY ? 0.f : mx;  // nothing visible yet: every weight below is 2^-inf = 0
    const float old = __builtin_amdgcn_exp2f(m - ref);
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < NS; ++t)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[t][i] = __builtin_amdgcn_exp2f(s[t][i] - ref);
        sum += s[t][i];
      }
    sum += __shfl_xor(sum, 16);
    sum += __shfl_xor(sum, 32);
    l = l * old + sum;
    m = mx;
#pragma unroll
    for (int i = 0; i < VTL; ++i) {
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
// calls f with the smallest instantiated (KT, VTL) that holds kts k tiles and vts value tiles
template <typename F>
static int attn_sizes(int kts, int vts, F&& f, const char* what) {
  if (kts <= 2 && vts <= 4) return f(std::integral_constant<int, 2>{}, std::integral_constant<int, 4>{});
  if (kts <= 4 && vts <= 8) return f(std::integral_constant<int, 4>{}, std::integral_constant<int, 8>{});
  if (kts <= 6 && vts <= 8) return f(std::integral_constant<int, 6>{}, std::integral_constant<int, 8>{});
  if (kts <= 8 && vts <= 16) return f(std::integral_constant<int, 8>{}, std::integral_constant<int, 16>{});
  DSK_FAIL(DSK_ERR_UNSUPPORTED, "%s: key size %d, value size %d (max 256)", what, 32 * kts, 16 * vts);
}
#define ATTN_KERNEL(T) __global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(sizeof(T) == 2 ? 2 : 1, sizeof(T) == 2 ? 2 : 1)))
