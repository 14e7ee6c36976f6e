// kernels_mix_few.hip -- decode steps of layered models: the mixers of one layer and the router's choice in ONE launch of 16-wave
// workgroups, one kind of work per workgroup:
//   attention   (sequence, key head, 256 keys of the chunk): rotation and norms of the new token's q and k, scores, weights, values;
//               the last of a (sequence, key head)'s workgroups to arrive merges the parts
//   mLSTM       (sequence, head): gates, one step of the recurrence, norm, output gate
//   delta rule  (sequence, head): convolution, low-rank second halves, unit norms, decays, one step, norm, output gate
//   wkv         (sequence, head): low-rank second half and decays, one step with the current token's bonus, norm, output gate
//   router      one workgroup for the whole step
// Same formulas and the same roundings to the activation type as the prompt kernels (kernels_chunk_attn.hip, kernels_recur.hip).
#include "layered_kernels.h"
#include "route_device.h"
#include "seq_device.h"

#include <math.h>

#include <algorithm>

static int cdiv(int a, int b) { return (a + b - 1) / b; }

enum { NT = 1024, NW = 16 };

template <typename T>
DEV void load8(const T* p, float (&v)[8]) {
  const typename Frag<T>::type f = *reinterpret_cast<const typename Frag<T>::type*>(p);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = (float)f[e];
}

// ---- attention -------------------------------------------------------------------------------------------
// one wave: a head's rotated, normed vector (rounded to T) into LDS as floats, and optionally to global memory
template <typename T>
DEV void rot_norm(const ChunkAttnArgs& a, const T* src, float pos, float* dst, T* store) {
  const int lane = threadIdx.x & 63;
  float u[2], v[2], ss = 0.f;
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
      const T x = (T)(u[i] * r), y = (T)(v[i] * r);
      dst[2 * pr] = (float)x;
      dst[2 * pr + 1] = (float)y;
      if (store) {
        store[2 * pr] = x;
        store[2 * pr + 1] = y;
      }
    }
  }
}
DEV void put(float* p, float v) { __hip_atomic_store(p, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
DEV float take(const float* p) { return __hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }

static size_t attn_few_lds(const ChunkAttnArgs& a) {
  const int rep = a.heads / a.kv_heads;
  return ((size_t)(rep + 1) * a.dim_p + (size_t)rep * ATTN_SPLIT_KEYS + a.vdim_p + (2 * rep + 3) / 4 * 4 + (size_t)NW * 4 * a.vdim_p + 4) * 4;
}
template <typename T>
DEV void attn_few(const MixFewArgs& f, int b, float* lds) {
  const ChunkAttnArgs& a = f.attn;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int split = b % f.splits, g = b / f.splits % a.kv_heads, row = b / f.splits / a.kv_heads;
  const SeqDesc sq = a.p.seqs[row];
  const int pos = sq.pos0, first = pos / a.chunk * a.chunk;
  const int n_splits = (pos - first) / ATTN_SPLIT_KEYS + 1;
  if (split >= n_splits) return;
  const int k0 = first + split * ATTN_SPLIT_KEYS, n = min((int)ATTN_SPLIT_KEYS, pos + 1 - k0);
  const int rep = a.heads / a.kv_heads;
  float* sq_ = lds;                               // [rep][dim_p]
  float* knew = sq_ + (size_t)rep * a.dim_p;      // [dim_p]
  float* sc = knew + a.dim_p;                     // [rep][ATTN_SPLIT_KEYS]
  float* vnew = sc + (size_t)rep * ATTN_SPLIT_KEYS;  // [vdim_p]
  float* ml = vnew + a.vdim_p;                    // [rep][2]
  float* red = ml + (2 * rep + 3) / 4 * 4;        // [NW][4][vdim_p]
  unsigned* last = reinterpret_cast<unsigned*>(red + (size_t)NW * 4 * a.vdim_p);
  const T* P = reinterpret_cast<const T*>(a.proj_t) + (size_t)row * a.ld;
  T* ck = reinterpret_cast<T*>(sq.state + a.off_k);
  T* cv = reinterpret_cast<T*>(sq.state + a.off_v);
  const bool newest = split == n_splits - 1;      // this part holds the new token's key
  // this thread's keys and values, requested before anything else: 16 lanes per key, 8 elements per lane (twice past 128);
  // of the values a lane takes 4 channels of every (NW * kpw)-th key
  typedef typename Frag<T>::type frag;
  typedef typename Frag<T>::four four;
  constexpr int KI = ATTN_SPLIT_KEYS / (4 * NW);
  const int l16 = lane & 15;
  frag kr[KI][2];
#pragma unroll
  for (int u = 0; u < KI; ++u)
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int j = wave * 4 + (lane >> 4) + u * 4 * NW, e = l16 * 8 + 128 * i;
      kr[u][i] = frag{};
      if (j < n && k0 + j < pos && e < a.dim_p) kr[u][i] = *reinterpret_cast<const frag*>(ck + ((size_t)((k0 + j) % a.chunk) * a.kv_heads + g) * a.dim_p + e);
    }
  const int nv4 = a.vdim_p >> 2;
  const int nvp = nv4 <= 8 ? 8 : nv4 <= 16 ? 16 : nv4 <= 32 ? 32 : 64, kpw = 64 / nvp;
  const int c4 = lane & (nvp - 1), kg = wave * kpw + lane / nvp;
  constexpr int VI = ATTN_SPLIT_KEYS / NW;  // values per thread at kpw = 1
  four vr[VI];
#pragma unroll
  for (int u = 0; u < VI; ++u) {
    const int j = kg + u * NW * kpw;
    vr[u] = four{};
    if (j < n && k0 + j < pos && c4 < nv4) vr[u] = *reinterpret_cast<const four*>(cv + ((size_t)((k0 + j) % a.chunk) * a.kv_heads + g) * a.vdim_p + 4 * c4);
  }
  for (int r = wave; r < rep; r += NW) rot_norm<T>(a, P + a.col_q + (g * rep + r) * a.dim, (float)pos, sq_ + (size_t)r * a.dim_p, nullptr);
  if (newest) {
    const size_t at = (size_t)(pos % a.chunk) * a.kv_heads + g;
    if (wave == NW - 1) rot_norm<T>(a, P + a.col_k + g * a.dim, (float)pos, knew, ck + at * a.dim_p);
    if (wave == NW - 2)
      for (int i = lane; i < a.vdim_p; i += 64) {
        const T v = i < a.vdim ? P[a.col_v + g * a.vdim + i] : (T)0.f;
        vnew[i] = (float)v;
        cv[at * a.vdim_p + i] = v;
      }
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < KI; ++u) {
    const int j = wave * 4 + (lane >> 4) + u * 4 * NW;
    const bool in = j < n;
    float k[2][8];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int e = l16 * 8 + 128 * i;
      const bool fresh = k0 + j == pos && e < a.dim_p;
#pragma unroll
      for (int x = 0; x < 8; ++x) k[i][x] = fresh ? knew[e + x] : (float)kr[u][i][x];
    }
    for (int r = 0; r < rep; ++r) {
      float d = 0.f;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        const int e = l16 * 8 + 128 * i;
        if (e >= a.dim_p) continue;
#pragma unroll
        for (int x = 0; x < 8; ++x) d += k[i][x] * sq_[(size_t)r * a.dim_p + e + x];
      }
      d = row_sum(d);
      if (l16 == 0) sc[r * ATTN_SPLIT_KEYS + j] = in ? d * a.scale : -INFINITY;
    }
  }
  __syncthreads();
  for (int r = wave; r < rep; r += NW) {
    float s[ATTN_SPLIT_KEYS / 64], m = -INFINITY, l = 0.f;
#pragma unroll
    for (int i = 0; i < ATTN_SPLIT_KEYS / 64; ++i) {
      s[i] = sc[r * ATTN_SPLIT_KEYS + lane + 64 * i];
      m = fmaxf(m, s[i]);
    }
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) m = fmaxf(m, __shfl_xor(m, off));
#pragma unroll
    for (int i = 0; i < ATTN_SPLIT_KEYS / 64; ++i) {
      const float p = expf(s[i] - m);
      l += p;
      sc[r * ATTN_SPLIT_KEYS + lane + 64 * i] = (float)(T)p;
    }
    l = wave_sum(l);
    if (lane == 0) {
      ml[2 * r] = m;
      ml[2 * r + 1] = l;
    }
  }
  __syncthreads();
  const size_t pstride = a.vdim_p + 2;
  for (int r0 = 0; r0 < rep; r0 += 4) {
    const int rn = min(4, rep - r0);
    f32x4 acc[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (c4 < nv4)
#pragma unroll
      for (int u = 0; u < VI; ++u) {
        const int j = kg + u * NW * kpw;
        if (j >= n) break;
        const f32x4 v = k0 + j == pos ? *reinterpret_cast<const f32x4*>(vnew + 4 * c4) : __builtin_convertvector(vr[u], f32x4);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (r < rn) acc[r] += sc[(r0 + r) * ATTN_SPLIT_KEYS + j] * v;
      }
    for (int off = nvp; off < 64; off <<= 1)
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[r][e] += __shfl_xor(acc[r][e], off);
    if (lane < nv4)
#pragma unroll
      for (int r = 0; r < 4; ++r) *reinterpret_cast<f32x4*>(red + ((size_t)wave * 4 + r) * a.vdim_p + 4 * lane) = acc[r];
    __syncthreads();
    for (int i = tid; i < rn * a.vdim_p; i += NT) {
      const int r = i / a.vdim_p, c = i % a.vdim_p, h = g * rep + r0 + r;
      float o = 0.f;
#pragma unroll
      for (int w = 0; w < NW; ++w) o += red[((size_t)w * 4 + r) * a.vdim_p + c];
      if (n_splits == 1) {
        if (c < a.vdim) reinterpret_cast<T*>(a.out_t)[(size_t)row * a.out_ld + h * a.vdim + c] = (T)(o / ml[2 * (r0 + r) + 1]);
      } else {
        float* pt = f.part + (((size_t)row * a.heads + h) * f.splits + split) * pstride;
        put(pt + 2 + c, o);
        if (c < 2) put(pt + c, ml[2 * (r0 + r) + c]);
      }
    }
    __syncthreads();
  }
  if (n_splits == 1) return;
  // hand-off: drained write-through stores, one arrival; the last workgroup reads the parts with agent-scope loads
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (tid == 0) {
    unsigned* ctr = f.arrived + row * a.kv_heads + g;
    *last = __hip_atomic_fetch_add(ctr, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (unsigned)n_splits - 1;
    if (*last) {
      FINISHER_ACQUIRE();
      __hip_atomic_store(ctr, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    }
  }
  __syncthreads();
  if (!*last) return;
  // maxima and sums of all parts at once, then every output element adds its parts, eight loads in flight
  float *pm = red, *pl = red + rep * n_splits;
  const float* part0 = f.part + ((size_t)row * a.heads + g * rep) * f.splits * pstride;
  for (int i = tid; i < rep * n_splits; i += NT) {
    const float* pt = part0 + ((size_t)(i / n_splits) * f.splits + i % n_splits) * pstride;
    pm[i] = take(pt);
    pl[i] = take(pt + 1);
  }
  __syncthreads();
  for (int r = wave; r < rep; r += NW) {
    float m = -INFINITY, l = 0.f;
    for (int s = lane; s < n_splits; s += 64) m = fmaxf(m, pm[r * n_splits + s]);
#pragma unroll
    for (int off = 32; off >= 1; off >>= 1) m = fmaxf(m, __shfl_xor(m, off));
    for (int s = lane; s < n_splits; s += 64) {
      const float w = expf(pm[r * n_splits + s] - m);
      l += w * pl[r * n_splits + s];
      pm[r * n_splits + s] = w;
    }
    l = wave_sum(l);
    if (lane == 0) ml[2 * r + 1] = l;
  }
  __syncthreads();
  for (int i = tid; i < rep * a.vdim; i += NT) {
    const int r = i / a.vdim, c = i % a.vdim;
    const float* pt = part0 + (size_t)r * f.splits * pstride + 2 + c;
    float o = 0.f;
    for (int s0 = 0; s0 < n_splits; s0 += 8) {
      float v[8];
#pragma unroll
      for (int u = 0; u < 8; ++u) v[u] = take(pt + min(s0 + u, n_splits - 1) * pstride);
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (s0 + u < n_splits) o += pm[r * n_splits + s0 + u] * v[u];
    }
    reinterpret_cast<T*>(a.out_t)[(size_t)row * a.out_ld + (g * rep + r) * a.vdim + c] = (T)(o / ml[2 * r + 1]);
  }
}

// ---- recurrent heads: how a workgroup holds a head's state [dim][vdim] ----------------------------------------
// Waves are dealt to groups of 64 columns and to ranges of key channels; a lane keeps RK channels of one column.
struct HeadTile {
  int col, k0, kn, parts;  // this lane's column, its channels [k0, k0 + kn), ranges a column is cut into
  bool on;
};
DEV HeadTile head_tile(int dim, int vdim) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int groups = (vdim + 63) >> 6, parts = NW / groups, per = (dim + parts - 1) / parts;
  HeadTile t;
  const int part = wave / groups;
  t.col = wave % groups * 64 + lane;
  t.k0 = part * per;
  t.kn = max(0, min(per, dim - t.k0));
  t.parts = parts;
  t.on = part < parts && t.col < vdim;
  return t;
}
static int head_rk(int dim, int vdim) {  // channels a lane holds
  const int parts = NW / cdiv(vdim, 64);
  return cdiv(dim, parts);
}
template <int RK>
DEV void load_state(const float* S0, const HeadTile& t, int vdim, bool fresh, float (&S)[RK]) {
#pragma unroll
  for (int i = 0; i < RK; ++i) S[i] = !fresh && t.on && i < t.kn ? S0[(size_t)(t.k0 + i) * vdim + t.col] : 0.f;
}
template <int RK>
DEV void store_state(float* S0, const HeadTile& t, int vdim, const float (&S)[RK]) {
#pragma unroll
  for (int i = 0; i < RK; ++i)
    if (t.on && i < t.kn) S0[(size_t)(t.k0 + i) * vdim + t.col] = S[i];
}
// behind the recurrence: o[vdim] in LDS -> RMS norm, weight, gate
template <typename T, typename G>
DEV void head_out(const float* o, int vdim, float eps, const float* w, G gate, T* out) {
  float ss = 0.f;
  for (int i = threadIdx.x & 63; i < vdim; i += 64) ss += o[i] * o[i];
  ss = wave_sum(ss);  // (every wave for itself)
  const float r = 1.f / sqrtf(ss / vdim + eps);
  for (int i = threadIdx.x; i < vdim; i += NT) out[i] = (T)(o[i] * r * w[i] * gate(i));
}

enum { HD = RECUR_MAX_DIM };
template <typename T, int RK>
DEV void mlstm_few(const MlstmArgs& a, int b, float* lds) {
  const int tid = threadIdx.x, lane = tid & 63;
  const int h = b % a.heads, row = b / a.heads;
  const SeqDesc s = a.p.seqs[row];
  const bool fresh = s.pos0 == 0;
  float *q = lds, *k = q + HD, *v = k + HD, *o = v + HD, *red = o + HD;  // red [16][HD]
  float* S0 = reinterpret_cast<float*>(s.state + a.off_s) + (size_t)h * a.dim * a.vdim;
  const HeadTile t = head_tile(a.dim, a.vdim);
  float S[RK];
  load_state<RK>(S0, t, a.vdim, fresh, S);
  const T* P = reinterpret_cast<const T*>(a.proj_t) + (size_t)row * a.ld;
  const float* G = a.gate_f + (size_t)row * a.ld_gate;
  for (int i = tid; i < a.dim; i += NT) {
    q[i] = (float)P[a.col_q + h * a.dim + i] * a.q_scale;
    k[i] = (float)P[a.col_k + h * a.dim + i];
  }
  for (int i = tid; i < a.vdim; i += NT) v[i] = (float)P[a.col_v + h * a.vdim + i];
  const float* N0 = reinterpret_cast<const float*>(s.state + a.off_n) + (size_t)h * a.dim + (size_t)s.flip * a.heads * a.dim;
  float* N1 = reinterpret_cast<float*>(s.state + a.off_n) + (size_t)h * a.dim + (size_t)(s.flip ^ 1) * a.heads * a.dim;
  float* M = reinterpret_cast<float*>(s.state + a.off_m) + h;
  const float gi = a.gate_cap * tanhf((G[a.col_i + h] + a.b_i[h]) / a.gate_cap);
  const float gf = logsigmoid_f(a.gate_cap * tanhf((G[a.col_f + h] + a.b_f[h]) / a.gate_cap));
  const float m0 = fresh ? 0.f : M[s.flip * a.heads];
  const float m = fmaxf(gf + m0, gi), keep = expf(gf + m0 - m), add = expf(gi - m);
  __syncthreads();
  float nq = 0.f;
  for (int i = lane; i < a.dim; i += 64) {
    const float n = keep * (fresh ? 0.f : N0[i]) + add * k[i];
    nq += n * q[i];
    if (tid < 64) N1[i] = n;
  }
  nq = wave_sum(nq);
  if (tid == 0) M[(s.flip ^ 1) * a.heads] = m;
  float p = 0.f;
  const float av = t.on ? add * v[t.col] : 0.f;
#pragma unroll
  for (int i = 0; i < RK; ++i)
    if (i < t.kn) {
      S[i] = keep * S[i] + av * k[t.k0 + i];
      p += S[i] * q[t.k0 + i];
    }
  store_state<RK>(S0, t, a.vdim, S);
  const int per = (a.dim + t.parts - 1) / t.parts, used = (a.dim + per - 1) / per;
  if (t.on && t.kn) red[(size_t)(t.k0 / per) * HD + t.col] = p;
  __syncthreads();
  if (tid < a.vdim) {
    float sum = 0.f;
    for (int i = 0; i < used; ++i) sum += red[(size_t)i * HD + tid];
    o[tid] = sum / (fmaxf(fabsf(nq), expf(-m)) + a.floor_eps);
  }
  __syncthreads();
  head_out<T>(o, a.vdim, a.eps, a.out_norm + h * a.vdim, [&](int i) { return sigmoid_f((float)P[a.col_g + h * a.vdim + i]); },
              reinterpret_cast<T*>(a.out_t) + (size_t)row * a.out_ld + h * a.vdim);
}

// second half of a low-rank pair out of LDS: 256 rows at a time, four threads per row share its columns; sums in red[4][2 HD].
// row_of(r): the row of low_w; groups(r, g0, g1): its groups of 8 columns that are not zero
template <typename T, typename R, typename G>
DEV void low_rank(const MixFewArgs& f, const float* low, float* red, int nr, R row_of, G groups) {
  const int tid = threadIdx.x;
  for (int r0 = 0; r0 < nr; r0 += 256) {
    const int r = r0 + (tid & 255);
    if (r >= nr) continue;
    const int R_ = row_of(r);
    int g0, g1;
    groups(r, g0, g1);
    const bf16* w = reinterpret_cast<const bf16*>(f.low_w) + (size_t)(R_ >> 4) * f.low_kt * 512 + (R_ & 15) * 8;
    float z = 0.f;
#pragma unroll 4
    for (int gr = g0 + (tid >> 8); gr < g1; gr += 4) {
      float x[8];
      load8<bf16>(w + (size_t)(gr >> 2) * 512 + (gr & 3) * 128, x);
#pragma unroll
      for (int e = 0; e < 8; ++e) z += x[e] * low[gr * 8 + e];
    }
    red[(tid >> 8) * 2 * HD + r] = z;
  }
}
DEV float low_sum(const float* red, int r) { return (red[r] + red[2 * HD + r]) + (red[4 * HD + r] + red[6 * HD + r]); }

template <typename T, int RK>
DEV void wkv_few(const MixFewArgs& f, int b, float* lds) {
  const WkvArgs& a = f.wkv;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, dim = a.dim;
  const int h = b % a.heads, row = b / a.heads;
  const SeqDesc s = a.p.seqs[row];
  float *r = lds, *k = r + HD, *v = k + HD, *w = v + HD, *o = w + HD, *bonus = o + HD, *low = bonus + 4;
  float* red = low + f.low_kt * 32;  // [16][HD], before that [4][2 HD]
  float* S0 = reinterpret_cast<float*>(s.state + a.off_s) + (size_t)h * dim * dim;
  const HeadTile t = head_tile(dim, dim);
  float S[RK];
  load_state<RK>(S0, t, dim, s.pos0 == 0, S);
  const T* P = reinterpret_cast<const T*>(a.proj_t) + (size_t)row * a.ld + h * dim;
  for (int i = tid; i < f.low_kt * 32; i += NT) low[i] = i < f.low_a ? f.wkv_low[(size_t)row * f.wkv_low_ld + i] : 0.f;
  for (int i = tid; i < dim; i += NT) {
    r[i] = (float)P[a.col_r + i];
    k[i] = (float)P[a.col_k + i];
    v[i] = (float)P[a.col_v + i];
  }
  __syncthreads();
  low_rank<T>(f, low, red, dim, [&](int i) { return h * dim + i; }, [&](int, int& g0, int& g1) {
    g0 = 0;
    g1 = (f.low_a + 7) >> 3;
  });
  if (wave == NW - 1) {
    float z = 0.f;
    for (int i = lane; i < dim; i += 64) z += r[i] * a.u[h * dim + i] * k[i];
    z = wave_sum(z);
    if (lane == 0) bonus[0] = z;
  }
  __syncthreads();
  for (int i = tid; i < dim; i += NT) w[i] = expf(-expf(low_sum(red, i) + a.w0[h * dim + i]));
  __syncthreads();
  float z = 0.f;
  const float vc = t.on ? v[t.col] : 0.f;
#pragma unroll
  for (int i = 0; i < RK; ++i)
    if (i < t.kn) {
      z += S[i] * r[t.k0 + i];
      S[i] = w[t.k0 + i] * S[i] + k[t.k0 + i] * vc;
    }
  store_state<RK>(S0, t, dim, S);
  const int per = (dim + t.parts - 1) / t.parts, used = (dim + per - 1) / per;
  if (t.on && t.kn) red[(size_t)(t.k0 / per) * HD + t.col] = z;
  __syncthreads();
  if (tid < dim) {
    float sum = bonus[0] * v[tid];
    for (int i = 0; i < used; ++i) sum += red[(size_t)i * HD + tid];
    o[tid] = sum;
  }
  __syncthreads();
  head_out<T>(o, dim, a.eps, a.out_norm + h * dim, [&](int i) { return silu_f((float)P[a.col_g + i]); }, reinterpret_cast<T*>(a.out_t) + (size_t)row * a.out_ld + h * dim);
}

template <typename T, int RK>
DEV void delta_few(const MixFewArgs& f, int b, float* lds) {
  const DeltaArgs& a = f.delta;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = b % a.heads, row = b / a.heads, rep = a.heads / a.kv_heads, kv = h / rep;
  const SeqDesc s = a.p.seqs[row];
  const bool fresh = s.pos0 == 0;
  const int dim = a.dim, vdim = a.vdim, nq = a.kv_heads * dim, nv = a.heads * vdim, C = 2 * nq + nv, taps = a.taps;
  float *ch = lds, *g = ch + 3 * HD, *gate = g + HD, *o = gate + HD, *sc = o + HD, *low = sc + 4;
  float* red = low + f.low_kt * 32;  // [16][2][HD], before that [4][2 HD]
  float *q = ch, *k = ch + HD, *v = ch + 2 * HD;
  float* S0 = reinterpret_cast<float*>(s.state + a.off_s) + (size_t)h * dim * vdim;
  const HeadTile t = head_tile(dim, vdim);
  float S[RK];
  load_state<RK>(S0, t, vdim, fresh, S);
  const T* P = reinterpret_cast<const T*>(a.proj_t) + (size_t)row * a.ld;
  for (int i = tid; i < f.low_kt * 32; i += NT) low[i] = i < f.low_a + f.low_g ? (float)P[f.col_low + i] : 0.f;
  {  // convolution + silu, and the inputs kept for the next token (q and k channels: the first head of a group keeps them)
    const float* hist = reinterpret_cast<const float*>(s.state + a.off_conv) + (size_t)s.flip * (taps - 1) * C;
    float* next = reinterpret_cast<float*>(s.state + a.off_conv) + (size_t)(s.flip ^ 1) * (taps - 1) * C;
    for (int i = tid; i < 2 * dim + vdim; i += NT) {
      const int part = i < dim ? 0 : i < 2 * dim ? 1 : 2, e = i - part * dim;
      const int c = part == 2 ? 2 * nq + h * vdim + e : part * nq + kv * dim + e;
      const float x = (float)P[part == 0 ? a.col_q + kv * dim + e : part == 1 ? a.col_k + kv * dim + e : a.col_v + h * vdim + e];
      const bool keep = part == 2 || h % rep == 0;
      float y = x * a.conv_w[(size_t)c * taps + taps - 1];
      for (int j = 0; j < taps - 1; ++j) {
        const float old = s.pos0 - (taps - 1) + j >= 0 ? hist[(size_t)j * C + c] : 0.f;
        y += old * a.conv_w[(size_t)c * taps + j];
        if (keep && j > 0) next[(size_t)(j - 1) * C + c] = old;
      }
      if (keep && taps > 1) next[(size_t)(taps - 2) * C + c] = x;
      ch[part * HD + e] = silu_f(y);
    }
  }
  __syncthreads();
  const int nr = a.head_decay ? 0 : dim + vdim;
  low_rank<T>(f, low, red, nr, [&](int r) { return r < dim ? h * dim + r : a.heads * dim + h * vdim + r - dim; },
              [&](int r, int& g0, int& g1) {
                g0 = r < dim ? 0 : f.low_a >> 3;
                g1 = r < dim ? (f.low_a + 7) >> 3 : (f.low_a + f.low_g + 7) >> 3;
              });
  if (wave < 3) {  // |q|^2, |k|^2, k . q
    const float *x = wave == 0 ? q : k, *y = wave == 1 ? k : q;
    float ss = 0.f;
    for (int i = lane; i < dim; i += 64) ss += x[i] * y[i];
    ss = wave_sum(ss);
    if (lane == 0) sc[wave] = ss;
  }
  __syncthreads();
  const float qr = a.q_scale / sqrtf(sc[0] + a.unit_eps), kr = 1.f / sqrtf(sc[1] + a.unit_eps);
  for (int r = tid; r < nr; r += NT) {
    const float z = low_sum(red, r);
    if (r < dim) g[r] = expf(-a.a_rate[h] * softplus_f(z + a.dt_bias[h * dim + r]));
    else gate[r - dim] = sigmoid_f(z);
  }
  if (a.head_decay) {
    const float d = expf(-a.a_rate[h] * softplus_f(a.gate_f[(size_t)row * a.ld_gate + a.col_a + h] + a.dt_bias[h]));
    for (int r = tid; r < dim; r += NT) g[r] = d;
    for (int r = tid; r < vdim; r += NT) gate[r] = silu_f((float)P[a.col_g + h * vdim + r]);
  }
  const float beta = sigmoid_f(a.gate_f[(size_t)row * a.ld_gate + a.col_b + h]);
  __syncthreads();
  const int per = (dim + t.parts - 1) / t.parts, used = (dim + per - 1) / per, part = t.k0 / per;
  float p = 0.f, r = 0.f;
#pragma unroll
  for (int i = 0; i < RK; ++i)
    if (i < t.kn) {
      S[i] *= g[t.k0 + i];
      p += S[i] * (k[t.k0 + i] * kr);
      r += S[i] * (q[t.k0 + i] * qr);
    }
  if (t.on && t.kn) {
    red[(size_t)part * 2 * HD + t.col] = p;
    red[(size_t)part * 2 * HD + HD + t.col] = r;
  }
  __syncthreads();
  if (t.on) {
    float ps = 0.f, rs = 0.f;
    for (int i = 0; i < used; ++i) {
      ps += red[(size_t)i * 2 * HD + t.col];
      rs += red[(size_t)i * 2 * HD + HD + t.col];
    }
    const float u = beta * (v[t.col] - ps);
#pragma unroll
    for (int i = 0; i < RK; ++i)
      if (i < t.kn) S[i] += k[t.k0 + i] * kr * u;
    if (t.k0 == 0) o[t.col] = rs + sc[2] * kr * qr * u;
  }
  store_state<RK>(S0, t, vdim, S);
  __syncthreads();
  head_out<T>(o, vdim, a.eps, a.out_norm, [&](int i) { return gate[i]; }, reinterpret_cast<T*>(a.out_t) + (size_t)row * a.out_ld + h * vdim);
}

template <typename T, int RK>
__global__ __launch_bounds__(NT) void mix_few_kernel(const MixFewArgs f) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  int b = blockIdx.x;
  if (f.has_delta) {
    if (b < f.rows * f.delta.heads) {
      delta_few<T, RK>(f, b, lds);
      return;
    }
    b -= f.rows * f.delta.heads;
  }
  if (f.has_mlstm) {
    if (b < f.rows * f.mlstm.heads) {
      mlstm_few<T, RK>(f.mlstm, b, lds);
      return;
    }
    b -= f.rows * f.mlstm.heads;
  }
  if (f.has_wkv) {
    if (b < f.rows * f.wkv.heads) {
      wkv_few<T, RK>(f, b, lds);
      return;
    }
    b -= f.rows * f.wkv.heads;
  }
  if (f.has_route) {
    if (b == 0) {
      route_few_body(f.moe, reinterpret_cast<char*>(lds));
      return;
    }
    b -= 1;
  }
  attn_few<T>(f, b, lds);
}

// ---- launch ---------------------------------------------------------------------------------------------------
static size_t mix_lds(const MixFewArgs& f) {
  size_t n = ROUTE_FEW_LDS;
  if (f.has_attn) n = std::max(n, attn_few_lds(f.attn));
  if (f.has_mlstm) n = std::max(n, (size_t)(4 + NW) * HD * 4);
  if (f.has_delta) n = std::max(n, ((size_t)(6 + 2 * NW) * HD + 4 + f.low_kt * 32) * 4);
  if (f.has_wkv) n = std::max(n, ((size_t)(5 + NW) * HD + 4 + f.low_kt * 32) * 4);
  return n;
}
bool mix_few_fits(const MixFewArgs& f) {
  if (f.has_attn && (f.attn.dim > 256 || f.attn.vdim > 256 || (f.attn.dim & 1))) return false;
  if (f.has_attn && 2 * f.attn.heads / f.attn.kv_heads * f.splits > NW * 4 * f.attn.vdim_p) return false;  // (the merge's sums in LDS)
  if (f.has_mlstm && (f.mlstm.dim > HD || f.mlstm.vdim > HD)) return false;
  if (f.has_delta && (f.delta.dim > HD || f.delta.vdim > HD)) return false;
  if (f.has_wkv && f.wkv.dim > HD) return false;
  if (f.has_route && (f.moe.experts > ROUTE_MAX_EXPERTS || f.moe.top + f.moe.shared > 64)) return false;
  return f.rows <= 16 && mix_lds(f) <= 128 * 1024;
}
template <typename T, int RK>
static int mix_t(hipStream_t st, const MixFewArgs& f) {
  const size_t lds = mix_lds(f);
  const int grid = f.rows * ((f.has_delta ? f.delta.heads : 0) + (f.has_mlstm ? f.mlstm.heads : 0) + (f.has_wkv ? f.wkv.heads : 0) + (f.has_attn ? f.attn.kv_heads * f.splits : 0)) + (f.has_route ? 1 : 0);
  auto k = mix_few_kernel<T, RK>;
  HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(k), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  hipLaunchKernelGGL(k, dim3(grid), dim3(NT), lds, st, f);
  return DSK_OK;
}
template <typename T>
static int mix_rk(hipStream_t st, const MixFewArgs& f) {
  int rk = 1;
  if (f.has_mlstm) rk = std::max(rk, head_rk(f.mlstm.dim, f.mlstm.vdim));
  if (f.has_delta) rk = std::max(rk, head_rk(f.delta.dim, f.delta.vdim));
  if (f.has_wkv) rk = std::max(rk, head_rk(f.wkv.dim, f.wkv.dim));
  return rk <= 8 ? mix_t<T, 8>(st, f) : rk <= 16 ? mix_t<T, 16>(st, f) : rk <= 32 ? mix_t<T, 32>(st, f) : mix_t<T, 64>(st, f);
}
int launch_mix_few(hipStream_t st, const MixFewArgs& f, bool f32) {
  if (!mix_few_fits(f)) DSK_FAIL(DSK_ERR_UNSUPPORTED, "mix_few: sizes");
  return f32 ? mix_rk<float>(st, f) : mix_rk<bf16>(st, f);
}
