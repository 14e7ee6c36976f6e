// kernels_join.hip -- between the matrix products of layered models: the 32-bit residual sum with the norm behind it, the causal
// convolution and the blends with the previous token that may follow the norm, and the router's choice of experts.
#include "layered_kernels.h"
#include "route_device.h"
#include "seq_device.h"

#include <math.h>

// ---- residual + norm -----------------------------------------------------------------------------
// One workgroup per row; a thread keeps VPT groups of V consecutive elements in registers (V = 4, or 1 for widths that 4 does not divide).
template <typename S, int V>
DEV void load_v(const S* p, bool in, float (&v)[V]) {
  if constexpr (V == 4) {
    typedef S s4 __attribute__((ext_vector_type(4)));
    const s4 q = in ? *reinterpret_cast<const s4*>(p) : s4{};
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = (float)q[e];
  } else {
    v[0] = in ? (float)p[0] : 0.f;
  }
}
template <typename S, int V>
DEV void store_v(S* p, const float (&v)[V]) {
  if constexpr (V == 4) {
    typedef S s4 __attribute__((ext_vector_type(4)));
    *reinterpret_cast<s4*>(p) = s4{(S)v[0], (S)v[1], (S)v[2], (S)v[3]};
  } else {
    p[0] = (S)v[0];
  }
}
// A sequence's only token of the pass: V channels of h through the convolution.  TAPS = 4: what that needs from memory is requested at
// once, early enough to be there when h is (the blends' weights: up to MAX_MIX); TAPS = 1: any number of taps, one after the other.
template <int V, int TAPS>
struct ConvOne {
  enum { MAX_MIX = 5, KEPT = TAPS > 1 ? TAPS - 1 : 1, MIX = TAPS > 1 ? (int)MAX_MIX : 1 };
  float old[KEPT][V], w[V * TAPS], mu[MIX][V], prev[V];
  const float* hist;
  float *next, *p_next;
  DEV void load(const JoinArgs& j, const SeqDesc& s, int c) {
    const ConvArgs& a = j.conv;
    const int D = j.width, taps = TAPS > 1 ? TAPS : a.taps;
    hist = reinterpret_cast<const float*>(s.state + a.off_in) + (size_t)s.flip * (taps - 1) * D + c;
    next = reinterpret_cast<float*>(s.state + a.off_in) + (size_t)(s.flip ^ 1) * (taps - 1) * D + c;
    p_next = reinterpret_cast<float*>(s.state + a.off_prev) + c + (size_t)(s.flip ^ 1) * D;
    if (c >= D) return;
    if constexpr (TAPS > 1) {
#pragma unroll
      for (int t = 0; t < KEPT; ++t) load_v<float, V>(hist + (size_t)t * D, s.pos0 - (taps - 1) + t >= 0, old[t]);
#pragma unroll
      for (int e = 0; e < TAPS; ++e) load_v<float, V>(a.w + (size_t)c * taps + e * V, true, *reinterpret_cast<float(*)[V]>(w + e * V));
    }
    if (a.mu) {
      load_v<float, V>(reinterpret_cast<const float*>(s.state + a.off_prev) + c + (size_t)s.flip * D, s.pos0 > 0, prev);
      if constexpr (TAPS > 1) {
#pragma unroll
        for (int i = 0; i < MIX; ++i) load_v<float, V>(a.mu + (size_t)min(i, a.n_mix - 1) * D + c, true, mu[i]);
      }
    }
  }
  template <typename T>
  DEV void run(const JoinArgs& j, int row, int pos0, int c, const float (&h)[V]) {
    const ConvArgs& a = j.conv;
    const int D = j.width, taps = TAPS > 1 ? TAPS : a.taps;
    T* out = reinterpret_cast<T*>(a.out_t) + (size_t)row * a.ld + c;
    float y[V];
#pragma unroll
    for (int e = 0; e < V; ++e) y[e] = 0.f;
    if constexpr (TAPS > 1) {
#pragma unroll
      for (int t = 0; t < TAPS; ++t)
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] += (t == TAPS - 1 ? h[e] : old[t < KEPT ? t : 0][e]) * w[e * TAPS + t];
#pragma unroll
      for (int t = 1; t < KEPT; ++t) store_v<float, V>(next + (size_t)(t - 1) * D, old[t]);
    } else {
      for (int t = 0; t < taps - 1; ++t) {
        float o[V];
        load_v<float, V>(hist + (size_t)t * D, pos0 - (taps - 1) + t >= 0, o);
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] += o[e] * a.w[(size_t)(c + e) * taps + t];
        if (t > 0) store_v<float, V>(next + (size_t)(t - 1) * D, o);
      }
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] += h[e] * a.w[(size_t)(c + e) * taps + taps - 1];
    }
    if (taps > 1) store_v<float, V>(next + (size_t)(taps - 2) * D, h);
#pragma unroll
    for (int e = 0; e < V; ++e) y[e] += h[e];
    if (!a.mu) {
      store_v<T, V>(out, y);
      return;
    }
    store_v<float, V>(p_next, y);
    auto blend = [&](int i, const float (&m)[V]) {
      float v[V];
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = y[e] + (prev[e] - y[e]) * m[e];
      store_v<T, V>(out + i * a.mix_stride, v);
    };
    if constexpr (TAPS > 1) {
#pragma unroll
      for (int i = 0; i < MIX; ++i)
        if (i < a.n_mix) blend(i, mu[i]);
    } else {
      for (int i = 0; i < a.n_mix; ++i) {
        float m[V];
        load_v<float, V>(a.mu + (size_t)i * D + c, true, m);
        blend(i, m);
      }
    }
  }
};
// the sum of up to 8 rows, all requested at once (threads with many groups of elements: one row after the other)
template <int V, bool MANY>
struct LoadSum {
  float q[MANY ? 1 : 8][V];
  DEV void load(const float* p, bool in, int parts, size_t stride) {
    if constexpr (MANY) {
      load_v<float, V>(p, in, q[0]);
#pragma unroll 1
      for (int u = 1; u < parts; ++u) {
        float w[V];
        load_v<float, V>(p + u * stride, in, w);
#pragma unroll
        for (int e = 0; e < V; ++e) q[0][e] += w[e];
      }
    } else {
#pragma unroll
      for (int u = 0; u < 8; ++u) load_v<float, V>(p + u * stride, in && u < max(parts, 1), q[u]);
    }
  }
  DEV void sum(float (&v)[V]) const {
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = MANY ? q[0][e] : ((q[0][e] + q[1][e]) + (q[2][e] + q[3][e])) + ((q[4][e] + q[5][e]) + (q[6][e] + q[7][e]));
  }
};
// CONV: taps of the convolution behind the norm (single tokens; ConvOne), 0: none
template <typename T, int NT, int VPT, int V, int CONV>
__global__ __launch_bounds__(NT) void join_kernel(const JoinArgs a) {
  __shared__ float red[NT / 64], s_w[64];
  __shared__ int s_pos[64];
  const int tid = threadIdx.x, D = a.width;
  const int row = a.only_want ? a.p.want[blockIdx.x] : (int)blockIdx.x;
  const int hrow = blockIdx.x;
  float x[VPT][V], add[VPT][V];
  auto at = [&](int i) { return V * (tid + i * NT); };
  // with a convolution behind the norm (single tokens: row = sequence): everything it reads and the norms' weights, requested behind the
  // sum's operands (one group per thread) or together with its use (more)
  ConvOne<V, (CONV > 1 ? CONV : 1)> cv;
  SeqDesc sq{};
  float nw[V], pw[V];
  if constexpr (CONV > 0) sq = a.p.seqs[row];
  if (a.y_t && tid < a.n_slots) {
    s_w[tid] = a.weight[(size_t)row * a.n_slots + tid];
    s_pos[tid] = a.slot_pos[(size_t)row * a.n_slots + tid];
  }
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    if (a.embed) load_v<bf16, V>(reinterpret_cast<const bf16*>(a.embed) + (size_t)a.p.tokens[row] * D + at(i), at(i) < D, x[i]);
    else load_v<float, V>(a.x + (size_t)row * D + at(i), at(i) < D, x[i]);
#pragma unroll
    for (int e = 0; e < V; ++e) add[i][e] = 0.f;
  }
  if constexpr (CONV > 0 && VPT == 1) {
    if (!a.mix_a) {
      load_v<float, V>(a.norm_w + at(0), at(0) < D, nw);
      cv.load(a, sq, at(0));
    }
  }
  if (a.mix_a) {
    const float* ma = a.mix_a + (size_t)row * a.mix_ld;
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      LoadSum<V, (VPT > 2)> q;
      q.load(ma + at(i), at(i) < D, a.parts_a, a.mix_stride);
      if constexpr (CONV > 0 && VPT == 1) {
        if (a.post_w) load_v<float, V>(a.post_w + at(0), at(0) < D, pw);
        load_v<float, V>(a.norm_w + at(0), at(0) < D, nw);
        cv.load(a, sq, at(0));
      }
      q.sum(add[i]);
    }
    if (a.mix_b) {
      const float* mb = a.mix_b + (size_t)row * a.mix_ld;
      float vb[VPT][V], sa = 0.f, sb = 0.f;
#pragma unroll
      for (int i = 0; i < VPT; ++i) {
        LoadSum<V, (VPT > 2)> q;
        q.load(mb + at(i), at(i) < D, a.parts_b, a.mix_stride);
        q.sum(vb[i]);
#pragma unroll
        for (int e = 0; e < V; ++e) {
          sa += add[i][e] * add[i][e];
          sb += vb[i][e] * vb[i][e];
        }
      }
      sa = block_sum<NT>(sa, red);
      sb = block_sum<NT>(sb, red);
      const float ra = 1.f / sqrtf(sa / D + a.eps), rb = 1.f / sqrtf(sb / D + a.eps);
#pragma unroll
      for (int i = 0; i < VPT; ++i) {
        float wa[V], wb[V];
        load_v<float, V>(a.pair_wa + at(i), at(i) < D, wa);
        load_v<float, V>(a.pair_wb + at(i), at(i) < D, wb);
#pragma unroll
        for (int e = 0; e < V; ++e) add[i][e] = 0.5f * (add[i][e] * ra * wa[e] + vb[i][e] * rb * wb[e]);
      }
    } else if (a.post_w) {
      float sa = 0.f;
#pragma unroll
      for (int i = 0; i < VPT; ++i)
#pragma unroll
        for (int e = 0; e < V; ++e) sa += add[i][e] * add[i][e];
      sa = block_sum<NT>(sa, red);
      const float ra = 1.f / sqrtf(sa / D + a.eps);
#pragma unroll
      for (int i = 0; i < VPT; ++i) {
        float w[V];
        if constexpr (CONV > 0 && VPT == 1) {
#pragma unroll
          for (int e = 0; e < V; ++e) w[e] = pw[e];
        } else {
          load_v<float, V>(a.post_w + at(i), at(i) < D, w);
        }
#pragma unroll
        for (int e = 0; e < V; ++e) add[i][e] *= ra * (w[e] + a.norm_offset);
      }
    }
  }
  if (a.y_t) {
    __syncthreads();
#pragma unroll 4
    for (int k = 0; k < a.n_slots; ++k) {
      const float w = s_w[k];
      const T* y = reinterpret_cast<const T*>(a.y_t) + (size_t)s_pos[k] * a.y_ld;
#pragma unroll
      for (int i = 0; i < VPT; ++i) {
        float v[V];
        load_v<T, V>(y + at(i), at(i) < D, v);
#pragma unroll
        for (int e = 0; e < V; ++e) add[i][e] += w * v[e];
      }
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
#pragma unroll
    for (int e = 0; e < V; ++e) {
      x[i][e] += add[i][e];
      ss += x[i][e] * x[i][e];
    }
    if (!a.only_want && at(i) < D) store_v<float, V>(a.x + (size_t)row * D + at(i), x[i]);
  }
  if (!a.norm_w) return;
  ss = block_sum<NT>(ss, red);
  const float r = 1.f / sqrtf(ss / D + a.eps);
  T* h = reinterpret_cast<T*>(a.h_t) + (size_t)hrow * a.h_ld;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    if (at(i) >= D) continue;
    float w[V];
    if constexpr (CONV > 0 && VPT == 1) {
#pragma unroll
      for (int e = 0; e < V; ++e) w[e] = nw[e];
    } else {
      if constexpr (CONV > 0) cv.load(a, sq, at(i));
      load_v<float, V>(a.norm_w + at(i), true, w);
    }
#pragma unroll
    for (int e = 0; e < V; ++e) w[e] = x[i][e] * r * (w[e] + a.norm_offset);
    if constexpr (CONV > 0) cv.template run<T>(a, row, sq.pos0, at(i), w);
    else if (a.h_f) store_v<float, V>(a.h_f + (size_t)row * D + at(i), w);
    else store_v<T, V>(h + at(i), w);
  }
}
template <typename T, int CONV>
static int join_t(hipStream_t st, const JoinArgs& a, int n) {
  const int D = a.width;
#define JOIN(NT, VPT, V) hipLaunchKernelGGL((join_kernel<T, NT, VPT, V, CONV>), dim3(n), dim3(NT), 0, st, a)
  if (D > 16384) DSK_FAIL(DSK_ERR_UNSUPPORTED, "join: width %d (max 16384)", D);
  if (D & 3) {
    if (D <= 1024) JOIN(256, 4, 1);
    else JOIN(1024, 16, 1);
  } else if (D <= 256) JOIN(64, 1, 4);
  else if (D <= 1024) JOIN(256, 1, 4);
  else if (D <= 2048) JOIN(512, 1, 4);
  else if (D <= 4096) JOIN(512, 2, 4);
  else if (D <= 8192) JOIN(1024, 2, 4);
  else JOIN(1024, 4, 4);
#undef JOIN
  return DSK_OK;
}
int launch_join(hipStream_t st, const JoinArgs& a, bool f32) {
  const int n = a.only_want ? a.p.n_want : a.p.rows;
  if (n < 1) DSK_FAIL(DSK_ERR_INVALID, "join: no rows");
  if (!a.conv.w) return f32 ? join_t<float, 0>(st, a, n) : join_t<bf16, 0>(st, a, n);
  if (a.conv.taps == 4 && a.conv.n_mix <= ConvOne<1, 4>::MAX_MIX) return f32 ? join_t<float, 4>(st, a, n) : join_t<bf16, 4>(st, a, n);
  return f32 ? join_t<float, 1>(st, a, n) : join_t<bf16, 1>(st, a, n);
}

// ---- convolution in front of a sublayer, portions --------------------------------------------------------
// y, or its blends with the previous token's y, of V channels from c on
template <typename T, int V>
DEV void store_blends(const ConvArgs& a, int D, int row, int c, const float (&y)[V], const float (&prev)[V]) {
  T* out = reinterpret_cast<T*>(a.out_t) + (size_t)row * a.ld + c;
  if (!a.mu) {
    store_v<T, V>(out, y);
    return;
  }
  for (int s = 0; s < a.n_mix; ++s) {
    float m[V];
    load_v<float, V>(a.mu + (size_t)s * D + c, true, m);
#pragma unroll
    for (int e = 0; e < V; ++e) m[e] = y[e] + (prev[e] - y[e]) * m[e];
    store_v<T, V>(out + s * a.mix_stride, m);
  }
}
// A thread takes V channels of the (up to 16) rows of a chunk; TAPS = 0: any number of taps, read from memory again and again.
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(256) void conv_kernel(const PassDesc p, int D, const float* __restrict__ h_f, const ConvArgs a) {
  constexpr int R = RECUR_CHUNK, K = TAPS ? TAPS : 1;
  const int c = V * (blockIdx.y * 256 + threadIdx.x), taps = TAPS ? TAPS : a.taps;
  if (c >= D) return;
  const SeqDesc s = p.seqs[p.chunk[2 * blockIdx.x]];
  const int t0 = p.chunk[2 * blockIdx.x + 1], n_rows = min(R, s.len - t0);
  const float* H = h_f + (size_t)s.row0 * D + c;
  const float* hist = reinterpret_cast<const float*>(s.state + a.off_in) + (size_t)s.flip * (taps - 1) * D + c;
  float* P = a.mu ? reinterpret_cast<float*>(s.state + a.off_prev) + c : nullptr;
  auto input = [&](int u, float (&v)[V]) {  // row u of the portion; before it: the kept inputs, zero before the sequence's start
    if (u >= 0) load_v<float, V>(H + (size_t)u * D, true, v);
    else load_v<float, V>(hist + (size_t)(max(u, 1 - taps) + taps - 1) * D, u >= 1 - taps && s.pos0 + u >= 0, v);
  };
  float y[V], prev[V];
  const bool has_prev = a.mu != nullptr;
  if constexpr (TAPS > 1) {
    float w[V][K], x[R + K][V];  // inputs t0 - taps .. t0 + 15 (the first one only for the previous token's y)
#pragma unroll
    for (int e = 0; e < V; ++e)
#pragma unroll
      for (int j = 0; j < K; ++j) w[e][j] = a.w[(size_t)(c + e) * K + j];
#pragma unroll
    for (int r = 0; r < R + K; ++r) input(min(t0 - K + r, s.len - 1), x[r]);
    auto conv = [&](int t, float (&out)[V]) {  // of input x[t + K]
#pragma unroll
      for (int e = 0; e < V; ++e) {
        float z = 0.f;
#pragma unroll
        for (int j = 0; j < K; ++j) z += x[t + 1 + j][e] * w[e][j];
        out[e] = x[t + K][e] + z;
      }
    };
    float ys[R + 1][V];  // behind the previous token's
    if (has_prev && t0 == 0) load_v<float, V>(P + (size_t)s.flip * D, s.pos0 > 0, ys[0]);
    else conv(-1, ys[0]);
#pragma unroll
    for (int t = 0; t < R; ++t) conv(t, ys[t + 1]);
    T* out = reinterpret_cast<T*>(a.out_t) + (size_t)(s.row0 + t0) * a.ld + c;
    for (int i = 0; i < (has_prev ? a.n_mix : 1); ++i) {
      float mu[V];
      load_v<float, V>(has_prev ? a.mu + (size_t)i * D + c : a.w, has_prev, mu);
#pragma unroll
      for (int t = 0; t < R; ++t) {
        float v[V];
#pragma unroll
        for (int e = 0; e < V; ++e) v[e] = ys[t + 1][e] + (ys[t][e] - ys[t + 1][e]) * mu[e];
        if (t < n_rows) store_v<T, V>(out + i * a.mix_stride + (size_t)t * a.ld, v);
      }
    }
#pragma unroll
    for (int t = 0; t < R; ++t)
#pragma unroll
      for (int e = 0; e < V; ++e)
        if (t < n_rows) y[e] = ys[t + 1][e];
  } else {
    auto conv = [&](int u, float (&out)[V]) {
      float x[V];
#pragma unroll
      for (int e = 0; e < V; ++e) out[e] = 0.f;
      for (int j = 0; j < taps; ++j) {
        input(u - (taps - 1) + j, x);
#pragma unroll
        for (int e = 0; e < V; ++e) out[e] += x[e] * a.w[(size_t)(c + e) * taps + j];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) out[e] += x[e];
    };
    if (has_prev) {
      if (t0 == 0) load_v<float, V>(P + (size_t)s.flip * D, s.pos0 > 0, prev);
      else conv(t0 - 1, prev);
    }
    for (int t = 0; t < n_rows; ++t) {
      conv(t0 + t, y);
      store_blends<T, V>(a, D, s.row0 + t0 + t, c, y, prev);
#pragma unroll
      for (int e = 0; e < V; ++e) prev[e] = y[e];
    }
  }
  if (t0 + n_rows < s.len) return;
  float* next = reinterpret_cast<float*>(s.state + a.off_in) + (size_t)(s.flip ^ 1) * (taps - 1) * D + c;
  for (int j = 0; j < taps - 1; ++j) {  // the portion's end: what the next one needs, in the other copy
    float x[V];
    input(s.len - (taps - 1) + j, x);
    store_v<float, V>(next + (size_t)j * D, x);
  }
  if (has_prev) store_v<float, V>(P + (size_t)(s.flip ^ 1) * D, y);
}
template <typename T, int V>
static void conv_t(hipStream_t st, const PassDesc& p, int D, const float* h_f, const ConvArgs& a) {
  const dim3 grid(p.n_chunks, (D / V + 255) / 256);
  switch (a.taps) {
    case 2: hipLaunchKernelGGL((conv_kernel<T, V, 2>), grid, dim3(256), 0, st, p, D, h_f, a); break;
    case 3: hipLaunchKernelGGL((conv_kernel<T, V, 3>), grid, dim3(256), 0, st, p, D, h_f, a); break;
    case 4: hipLaunchKernelGGL((conv_kernel<T, V, 4>), grid, dim3(256), 0, st, p, D, h_f, a); break;
    default: hipLaunchKernelGGL((conv_kernel<T, V, 0>), grid, dim3(256), 0, st, p, D, h_f, a);
  }
}
int launch_conv(hipStream_t st, const PassDesc& p, int width, const float* h_f, const ConvArgs& a, bool f32) {
  if (a.taps < 1 || width < 1 || p.n_chunks < 1) DSK_FAIL(DSK_ERR_INVALID, "conv: width %d, %d taps", width, a.taps);
  if (width & 3) f32 ? conv_t<float, 1>(st, p, width, h_f, a) : conv_t<bf16, 1>(st, p, width, h_f, a);
  else f32 ? conv_t<float, 4>(st, p, width, h_f, a) : conv_t<bf16, 4>(st, p, width, h_f, a);
  return DSK_OK;
}

// ---- router ----------------------------------------------------------------------------------------
__global__ __launch_bounds__(1024) void route_count_kernel(const MoeArgs a) {  // 16 rows per workgroup, one histogram
  __shared__ int hist[ROUTE_MAX_EXPERTS];
  const int tid = threadIdx.x, lane = tid & 63, ns = a.top + a.shared;
  for (int i = tid; i < a.experts; i += 1024) hist[i] = 0;
  __syncthreads();
  const int row = blockIdx.x * 16 + (tid >> 6);
  if (row < a.rows) {
    int e;
    float w;
    choose(a.logits + (size_t)row * a.ld_logits, a.experts, a.top, lane, &e, &w);
    if (lane < a.top) {
      a.chosen[(size_t)row * a.top + lane] = e;
      a.weight[(size_t)row * ns + lane] = w;
      atomicAdd(&hist[e], 1);
    } else if (lane == a.top && a.shared) {
      a.weight[(size_t)row * ns + lane] = 1.f;
    }
  }
  __syncthreads();
  for (int i = tid; i < a.experts; i += 1024)
    if (hist[i]) atomicAdd(a.count + i, hist[i]);
}
// offsets of the experts' slot ranges and the table of row tiles: one workgroup
__global__ __launch_bounds__(ROUTE_MAX_EXPERTS) void route_plan_kernel(const MoeArgs a) {
  __shared__ int off[ROUTE_MAX_EXPERTS + 1], til[ROUTE_MAX_EXPERTS + 1];
  const int e = threadIdx.x;
  const int n = e < a.experts ? a.count[e] : 0;
  off[e + 1] = n;
  til[e + 1] = (n + MOE_TILE - 1) / MOE_TILE;
  if (e == 0) off[0] = til[0] = 0;
  __syncthreads();
  for (int d = 1; d < ROUTE_MAX_EXPERTS; d <<= 1) {  // inclusive sums
    const int o = e + 1 > d ? off[e + 1 - d] : 0, t = e + 1 > d ? til[e + 1 - d] : 0;
    __syncthreads();
    off[e + 1] += o;
    til[e + 1] += t;
    __syncthreads();
  }
  if (e < a.experts) {
    a.cursor[e] = off[e];
    a.count[e] = 0;  // ready for the next layer
    for (int i = 0, t = til[e]; i < n; i += MOE_TILE, ++t) {
      a.tiles[4 * t] = e;
      a.tiles[4 * t + 1] = off[e] + i;
      a.tiles[4 * t + 2] = min(MOE_TILE, n - i);
    }
  }
  const int total = off[ROUTE_MAX_EXPERTS], t0 = til[ROUTE_MAX_EXPERTS];
  int n_tiles = t0;
  if (a.shared) {
    const int st = (a.rows + MOE_TILE - 1) / MOE_TILE;
    for (int i = e; i < st; i += ROUTE_MAX_EXPERTS) {
      a.tiles[4 * (t0 + i)] = a.experts;
      a.tiles[4 * (t0 + i) + 1] = total + i * MOE_TILE;
      a.tiles[4 * (t0 + i) + 2] = min(MOE_TILE, a.rows - i * MOE_TILE);
    }
    n_tiles += st;
  }
  if (e == 0) *a.n_tiles = n_tiles;
}
// one workgroup places 1024 slots: its slots of an expert are counted in LDS first and take one range of the expert's slots
__global__ __launch_bounds__(1024) void route_sort_kernel(const MoeArgs a) {
  __shared__ int n[ROUTE_MAX_EXPERTS], base[ROUTE_MAX_EXPERTS];
  const int tid = threadIdx.x, ns = a.top + a.shared;
  for (int i = tid; i < a.experts; i += 1024) n[i] = 0;
  __syncthreads();
  const int i = blockIdx.x * 1024 + tid;
  const bool in = i < a.rows * ns;
  const int row = i / ns, k = i % ns;
  int e = -1, at = 0;
  if (in && k < a.top) {
    e = a.chosen[(size_t)row * a.top + k];
    at = atomicAdd(&n[e], 1);
  }
  __syncthreads();
  for (int j = tid; j < a.experts; j += 1024)
    if (n[j]) base[j] = atomicAdd(a.cursor + j, n[j]);
  __syncthreads();
  if (!in) return;
  const int pos = e >= 0 ? base[e] + at : a.rows * a.top + row;
  a.slot_pos[i] = pos;
  a.slot_row[pos] = row;
}
__global__ __launch_bounds__(1024) void route_few_kernel(const MoeArgs a) {
  __shared__ __attribute__((aligned(16))) char lds[ROUTE_FEW_LDS];
  route_few_body(a, lds);
}
static int check_route(const MoeArgs& a) {
  if (a.experts < 1 || a.experts > ROUTE_MAX_EXPERTS || a.top < 1 || a.top > a.experts || a.top + a.shared > 64 || a.rows < 1)
    DSK_FAIL(DSK_ERR_UNSUPPORTED, "router: top %d of %d experts (at most 63 of %d)", a.top, a.experts, (int)ROUTE_MAX_EXPERTS);
  return DSK_OK;
}
int launch_route(hipStream_t st, const MoeArgs& a) {
  DSK_TRY(check_route(a));
  const int slots = a.rows * (a.top + a.shared);
  hipLaunchKernelGGL(route_count_kernel, dim3((a.rows + 15) / 16), dim3(1024), 0, st, a);
  hipLaunchKernelGGL(route_plan_kernel, dim3(1), dim3(ROUTE_MAX_EXPERTS), 0, st, a);
  hipLaunchKernelGGL(route_sort_kernel, dim3((slots + 1023) / 1024), dim3(1024), 0, st, a);
  return DSK_OK;
}
int launch_route_few(hipStream_t st, const MoeArgs& a) {
  DSK_TRY(check_route(a));
  if (a.rows > 16) DSK_FAIL(DSK_ERR_INVALID, "route_few: %d rows", a.rows);
  hipLaunchKernelGGL(route_few_kernel, dim3(1), dim3(1024), 0, st, a);
  return DSK_OK;
}
