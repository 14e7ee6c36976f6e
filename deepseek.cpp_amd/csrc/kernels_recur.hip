// kernels_recur.hip -- recurrent mixers of layered models: the gated delta rule with a decay per key channel or per head, mLSTM's
// matrix memory, and time mixing with a bonus for the current token (wkv).  Everything that enters the recurrence is computed in 32-bit; the state is 32-bit and lives in the sequence's arena.
//
// The columns of a head's state S [dim][vdim] never meet each other inside the recurrence, so a scan cuts a head into slices of 16
// columns: one workgroup of 4 waves per (slice, head, sequence), a wave holds 4 columns, 16 lanes share a column's dim key channels
// (KPL each, in registers).  Per token: two dot products over key channels (DPP sums over 16 lanes) and one rank-1 update.  The
// inputs of the next 16 tokens travel to registers while the current 16 are worked off from LDS.  (Passes of few long sequences run the
// recurrences chunk by chunk instead: kernels_chunk_scan.hip.)
#include "layered_kernels.h"
#include "seq_device.h"

#include <math.h>

static int cdiv(int a, int b) { return (a + b - 1) / b; }

// ---- delta rule: what enters the recurrence -----------------------------------------------------------
// A wave takes one unit for the (up to 16) rows of a chunk: a q or k head (short causal convolution, silu, unit norm), a v head
// (convolution, silu) or a head's decays and step sizes.  Lanes are channels; TAPS = 0: any number of taps, else that many in registers.
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void delta_prep_kernel(const DeltaArgs a) {
  constexpr int NI = RECUR_MAX_DIM / 64, R = RECUR_CHUNK;
  const int lane = threadIdx.x & 63, unit = blockIdx.y * 4 + (threadIdx.x >> 6);
  const int nq = a.kv_heads * a.dim, nv = a.heads * a.vdim, C = 2 * nq + nv, taps = TAPS ? TAPS : a.taps;
  if (unit >= 2 * a.kv_heads + 2 * a.heads) return;
  const SeqDesc sq = a.p.seqs[a.p.chunk[2 * blockIdx.x]];
  const int t0 = a.p.chunk[2 * blockIdx.x + 1], n_rows = min(R, sq.len - t0);
  const size_t row0 = (size_t)sq.row0 + t0;
  if (unit >= 2 * a.kv_heads + a.heads) {
    const int h = unit - 2 * a.kv_heads - a.heads;
    const float rate = a.a_rate[h];
    if (a.head_decay) {
      if (lane < n_rows) a.g[(row0 + lane) * a.heads + h] = expf(-rate * softplus_f(a.gate_f[(row0 + lane) * a.ld_gate + a.col_a + h] + a.dt_bias[h]));
    } else for (int i = lane; i < a.dim; i += 64) {
      const float bias = a.dt_bias[h * a.dim + i];
#pragma unroll 4
      for (int t = 0; t < n_rows; ++t)
        a.g[((row0 + t) * a.heads + h) * a.dim + i] = expf(-rate * softplus_f(a.low_f[(row0 + t) * a.ld_low + h * a.dim + i] + bias));
    }
    if (lane < n_rows) a.beta[(row0 + lane) * a.heads + h] = sigmoid_f(a.gate_f[(row0 + lane) * a.ld_gate + a.col_b + h]);
    return;
  }
  const bool is_v = unit >= 2 * a.kv_heads, is_q = unit < a.kv_heads;
  const int n = is_v ? a.vdim : a.dim;
  const int c0 = is_v ? 2 * nq + (unit - 2 * a.kv_heads) * a.vdim : unit * a.dim;              // first of the unit's C channels
  const int col = is_q ? a.col_q + c0 : is_v ? a.col_v + c0 - 2 * nq : a.col_k + c0 - nq;      // its column in the projections
  const T* P = reinterpret_cast<const T*>(a.proj_t) + (size_t)sq.row0 * a.ld + col;
  const float* hist = reinterpret_cast<const float*>(sq.state + a.off_conv) + (size_t)sq.flip * (taps - 1) * C + c0;
  auto input = [&](int u, int c) {  // row u of the portion; before it: the kept inputs, zero before the sequence's start
    if (u >= 0) return (float)P[(size_t)u * a.ld + c];
    return sq.pos0 + u >= 0 ? hist[(size_t)(u + taps - 1) * C + c] : 0.f;
  };
  float y[NI][R], ss[R];
#pragma unroll
  for (int t = 0; t < R; ++t) ss[t] = 0.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = lane + 64 * i;
#pragma unroll
    for (int t = 0; t < R; ++t) y[i][t] = 0.f;
    if (c >= n) continue;
    const float* w = a.conv_w + (size_t)(c0 + c) * taps;
    if constexpr (TAPS > 0) {
      float x[R + TAPS - 1];
#pragma unroll
      for (int r = 0; r < R + TAPS - 1; ++r) x[r] = input(min(t0 - (TAPS - 1) + r, sq.len - 1), c);
#pragma unroll
      for (int t = 0; t < R; ++t)
#pragma unroll
        for (int j = 0; j < TAPS; ++j) y[i][t] += x[t + j] * w[j];
    } else {
#pragma unroll
      for (int t = 0; t < R; ++t)
        if (t < n_rows)
          for (int j = 0; j < taps; ++j) y[i][t] += input(t0 + t - (taps - 1) + j, c) * w[j];
    }
#pragma unroll
    for (int t = 0; t < R; ++t) {
      y[i][t] = silu_f(y[i][t]);
      ss[t] += y[i][t] * y[i][t];
    }
  }
  float* dst = is_v ? a.v + row0 * nv + c0 - 2 * nq : is_q ? a.q + row0 * nq + c0 : a.k + row0 * nq + c0 - nq;
  const int ld = is_v ? nv : nq;
#pragma unroll
  for (int t = 0; t < R; ++t) {
    const float r = is_v ? 1.f : (is_q ? a.q_scale : 1.f) / sqrtf(wave_sum(ss[t]) + a.unit_eps);
#pragma unroll
    for (int i = 0; i < NI; ++i)
      if (t < n_rows && lane + 64 * i < n) dst[(size_t)t * ld + lane + 64 * i] = y[i][t] * r;
  }
  if (t0 + n_rows == sq.len) {  // the portion's end: keep the inputs of its last taps - 1 tokens, in the other copy
    float* next = reinterpret_cast<float*>(sq.state + a.off_conv) + (size_t)(sq.flip ^ 1) * (taps - 1) * C + c0;
    for (int j = 0; j < taps - 1; ++j)
      for (int c = lane; c < n; c += 64) next[(size_t)j * C + c] = input(sq.len - (taps - 1) + j, c);
  }
}
template <typename T>
static void delta_prep_t(hipStream_t st, const DeltaArgs& a) {
  const dim3 grid(a.p.n_chunks, cdiv(2 * a.kv_heads + 2 * a.heads, 4));
  switch (a.taps) {
    case 2: hipLaunchKernelGGL((delta_prep_kernel<T, 2>), grid, dim3(256), 0, st, a); break;
    case 3: hipLaunchKernelGGL((delta_prep_kernel<T, 3>), grid, dim3(256), 0, st, a); break;
    case 4: hipLaunchKernelGGL((delta_prep_kernel<T, 4>), grid, dim3(256), 0, st, a); break;
    default: hipLaunchKernelGGL((delta_prep_kernel<T, 0>), grid, dim3(256), 0, st, a);
  }
}
int launch_delta_prep(hipStream_t st, const DeltaArgs& a, bool f32) {
  if (a.dim > RECUR_MAX_DIM || a.vdim > RECUR_MAX_DIM) DSK_FAIL(DSK_ERR_UNSUPPORTED, "delta: key size %d, value size %d (max %d)", a.dim, a.vdim, (int)RECUR_MAX_DIM);
  if (f32) delta_prep_t<float>(st, a);
  else delta_prep_t<bf16>(st, a);
  return DSK_OK;
}

// ---- delta rule: the scan --------------------------------------------------------------------------
enum { SCAN_CH = 16 };  // tokens per LDS chunk
template <int KPL>
__global__ __launch_bounds__(256) void delta_scan_kernel(const DeltaArgs a) {
  constexpr int DK = 16 * KPL;  // padded dim
  __shared__ __attribute__((aligned(16))) float sq_[SCAN_CH][DK], sk_[SCAN_CH][DK], sg_[SCAN_CH][DK];
  __shared__ float sv_[SCAN_CH][16], sb_[SCAN_CH], skq[SCAN_CH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int kl = lane & 15, vl = wave * 4 + (lane >> 4);
  const int h = blockIdx.y, kv = h / (a.heads / a.kv_heads);
  const int col = blockIdx.x * 16 + vl;
  const bool live = col < a.vdim;
  const SeqDesc s = a.p.seqs[blockIdx.z];
  const int dim = a.dim, nq = a.kv_heads * dim, nv = a.heads * a.vdim;
  float* S0 = reinterpret_cast<float*>(s.state + a.off_s) + (size_t)h * dim * a.vdim;
  float S[KPL];
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const int k = kl * KPL + i;
    S[i] = s.pos0 > 0 && live && k < dim ? S0[(size_t)k * a.vdim + col] : 0.f;
  }
  // chunk loader: thread -> (token tid / 16, key channels (tid % 16) * KPL ..)
  const int lt = tid >> 4, lk = (tid & 15) * KPL;
  float rq[KPL], rk[KPL], rg[KPL], rv = 0.f, rb = 0.f;
  auto fetch = [&](int t0) {
    const int t = t0 + lt;
    const bool ok = t < s.len;
    const size_t row = (size_t)(s.row0 + (ok ? t : 0));
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      const bool in = ok && lk + i < dim;
      rq[i] = in ? a.q[row * nq + (size_t)kv * dim + lk + i] : 0.f;
      rk[i] = in ? a.k[row * nq + (size_t)kv * dim + lk + i] : 0.f;
      rg[i] = in ? (a.head_decay ? a.g[row * a.heads + h] : a.g[row * a.heads * dim + (size_t)h * dim + lk + i]) : 0.f;
    }
    const int c = blockIdx.x * 16 + (tid & 15);
    rv = ok && c < a.vdim ? a.v[row * nv + (size_t)h * a.vdim + c] : 0.f;
    rb = ok ? a.beta[row * a.heads + h] : 0.f;
  };
  fetch(0);
  for (int t0 = 0; t0 < s.len; t0 += SCAN_CH) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      sq_[lt][lk + i] = rq[i];
      sk_[lt][lk + i] = rk[i];
      sg_[lt][lk + i] = rg[i];
    }
    sv_[lt][tid & 15] = rv;
    float kq = 0.f;
#pragma unroll
    for (int i = 0; i < KPL; ++i) kq += rk[i] * rq[i];
    kq = row_sum(kq);
    if ((tid & 15) == 0) {
      sb_[lt] = rb;
      skq[lt] = kq;
    }
    __syncthreads();
    if (t0 + SCAN_CH < s.len) fetch(t0 + SCAN_CH);
    const int n = min((int)SCAN_CH, s.len - t0);
    float q[KPL], k[KPL], g[KPL];  // the current token's; the next one's are read while it is worked off
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      q[i] = sq_[0][kl * KPL + i];
      k[i] = sk_[0][kl * KPL + i];
      g[i] = sg_[0][kl * KPL + i];
    }
    float v = sv_[0][vl], b = sb_[0], c = skq[0];
    for (int t = 0; t < n; ++t) {
      const int t1 = min(t + 1, SCAN_CH - 1);
      float q1[KPL], k1[KPL], g1[KPL];
#pragma unroll
      for (int i = 0; i < KPL; ++i) {
        q1[i] = sq_[t1][kl * KPL + i];
        k1[i] = sk_[t1][kl * KPL + i];
        g1[i] = sg_[t1][kl * KPL + i];
      }
      const float v1 = sv_[t1][vl], b1 = sb_[t1], c1 = skq[t1];
      float p = 0.f, r = 0.f;
#pragma unroll
      for (int i = 0; i < KPL; ++i) {
        S[i] *= g[i];
        p += S[i] * k[i];
        r += S[i] * q[i];
      }
      p = row_sum(p);
      r = row_sum(r);
      const float u = b * (v - p);
#pragma unroll
      for (int i = 0; i < KPL; ++i) S[i] += k[i] * u;
      // S^T q behind the write = (decayed S)^T q + (k . q) u
      if (kl == 0 && live) a.o[(size_t)(s.row0 + t0 + t) * nv + (size_t)h * a.vdim + col] = r + c * u;
#pragma unroll
      for (int i = 0; i < KPL; ++i) {
        q[i] = q1[i];
        k[i] = k1[i];
        g[i] = g1[i];
      }
      v = v1;
      b = b1;
      c = c1;
    }
  }
  if (live)
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      const int k = kl * KPL + i;
      if (k < dim) S0[(size_t)k * a.vdim + col] = S[i];
    }
}
template <typename A, typename F>
static int by_kpl(const A& a, F&& f, const char* what) {  // key channels per lane: dim over 16 lanes, rounded up to an instantiation
  const int d = a.dim;
  if (d < 1 || d > RECUR_MAX_DIM) DSK_FAIL(DSK_ERR_UNSUPPORTED, "%s: key size %d (max %d)", what, d, (int)RECUR_MAX_DIM);
  return f(d <= 32 ? 2 : d <= 64 ? 4 : d <= 128 ? 8 : 16);
}
int launch_delta_scan(hipStream_t st, const DeltaArgs& a) {
  return by_kpl(a, [&](int kpl) {
    const dim3 grid(cdiv(a.vdim, 16), a.heads, a.p.n_seqs);
    if (kpl == 2) hipLaunchKernelGGL(delta_scan_kernel<2>, grid, dim3(256), 0, st, a);
    else if (kpl == 4) hipLaunchKernelGGL(delta_scan_kernel<4>, grid, dim3(256), 0, st, a);
    else if (kpl == 8) hipLaunchKernelGGL(delta_scan_kernel<8>, grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL(delta_scan_kernel<16>, grid, dim3(256), 0, st, a);
    return (int)DSK_OK;
  }, "delta");
}

// ---- behind a recurrence: per-head RMS norm, weight, gate ---------------------------------------------
// value(h, i): element i of head h; gate(c): the factor; w[c or i]: by place among all heads or inside one
template <typename T, typename V, typename G>
DEV void head_norm_gate(V value, int heads, int vdim, float eps, const float* w, bool shared_w, G gate, T* out) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  for (int h = wave; h < heads; h += 4) {
    float v[RECUR_MAX_DIM / 64], ss = 0.f;
#pragma unroll
    for (int i = 0; i < RECUR_MAX_DIM / 64; ++i) {
      v[i] = lane + 64 * i < vdim ? value(h, lane + 64 * i) : 0.f;
      ss += v[i] * v[i];
    }
    const float r = 1.f / sqrtf(wave_sum(ss) / vdim + eps);
#pragma unroll
    for (int i = 0; i < RECUR_MAX_DIM / 64; ++i) {
      const int e = lane + 64 * i, c = h * vdim + e;
      if (e < vdim) out[c] = (T)(v[i] * r * w[shared_w ? e : c] * gate(c));
    }
  }
}
template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(const DeltaArgs a) {
  const size_t row = blockIdx.x;
  const float *gl = a.low_f + row * a.ld_low + (size_t)a.heads * a.dim, *o = a.o + row * a.heads * a.vdim;
  const T* gp = reinterpret_cast<const T*>(a.proj_t) + row * a.ld + a.col_g;
  head_norm_gate<T>([&](int h, int i) { return o[h * a.vdim + i]; }, a.heads, a.vdim, a.eps, a.out_norm, true,
                    [&](int c) { return a.silu_gate ? silu_f((float)gp[c]) : sigmoid_f(gl[c]); }, reinterpret_cast<T*>(a.out_t) + row * a.out_ld);
}
int launch_delta_out(hipStream_t st, const DeltaArgs& a, bool f32) {
  if (f32) hipLaunchKernelGGL(delta_out_kernel<float>, dim3(a.p.rows), dim3(256), 0, st, a);
  else hipLaunchKernelGGL(delta_out_kernel<bf16>, dim3(a.p.rows), dim3(256), 0, st, a);
  return DSK_OK;
}
template <typename T, bool RAW>
__global__ __launch_bounds__(256) void mlstm_out_kernel(const MlstmArgs a, const float* __restrict__ floor_) {
  const size_t row = blockIdx.x;
  const int ld = RAW ? a.vdim + 1 : a.vdim;
  const float* o = a.o + row * a.heads * ld;
  const T* gl = reinterpret_cast<const T*>(a.proj_t) + row * a.ld + a.col_g;
  head_norm_gate<T>([&](int h, int i) {
    const float v = o[h * ld + i];
    return RAW ? v / (fmaxf(fabsf(o[h * ld + a.vdim]), floor_[row * a.heads + h]) + a.floor_eps) : v;
  }, a.heads, a.vdim, a.eps, a.out_norm, false, [&](int c) { return sigmoid_f((float)gl[c]); }, reinterpret_cast<T*>(a.out_t) + row * a.out_ld);
}
int launch_mlstm_out(hipStream_t st, const MlstmArgs& a, const ChunkScan* c, bool f32) {
  if (a.vdim > RECUR_MAX_DIM) DSK_FAIL(DSK_ERR_UNSUPPORTED, "mlstm: value size %d (max %d)", a.vdim, (int)RECUR_MAX_DIM);
  const float* fl = c ? c->floor : nullptr;
  const dim3 g(a.p.rows), b(256);
  if (f32 && c) hipLaunchKernelGGL((mlstm_out_kernel<float, true>), g, b, 0, st, a, fl);
  else if (f32) hipLaunchKernelGGL((mlstm_out_kernel<float, false>), g, b, 0, st, a, fl);
  else if (c) hipLaunchKernelGGL((mlstm_out_kernel<bf16, true>), g, b, 0, st, a, fl);
  else hipLaunchKernelGGL((mlstm_out_kernel<bf16, false>), g, b, 0, st, a, fl);
  return DSK_OK;
}

// ---- mLSTM: the scan ---------------------------------------------------------------------------------
// S and n carry the factor exp(-m) of the running maximum m; every slice keeps n and m for itself, slice 0 writes them back.
template <typename T, int KPL>
__global__ __launch_bounds__(256) void mlstm_scan_kernel(const MlstmArgs a) {
  constexpr int DK = 16 * KPL;
  __shared__ __attribute__((aligned(16))) float sq_[SCAN_CH][DK], sk_[SCAN_CH][DK];
  __shared__ float sv_[SCAN_CH][16], si_[SCAN_CH], sf_[SCAN_CH], s_keep[SCAN_CH], s_add[SCAN_CH], s_floor[SCAN_CH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int kl = lane & 15, vl = wave * 4 + (lane >> 4);
  const int h = blockIdx.y;
  const int col = blockIdx.x * 16 + vl;
  const bool live = col < a.vdim;
  const SeqDesc s = a.p.seqs[blockIdx.z];
  const int dim = a.dim, nv = a.heads * a.vdim;
  float* S0 = reinterpret_cast<float*>(s.state + a.off_s) + (size_t)h * dim * a.vdim;
  float* N0 = reinterpret_cast<float*>(s.state + a.off_n) + (size_t)h * dim;  // copy `flip` is read, the other written
  float* M0 = reinterpret_cast<float*>(s.state + a.off_m) + h;
  const int nn = a.heads * dim;
  float S[KPL], N[KPL], m = s.pos0 > 0 ? M0[s.flip * a.heads] : 0.f;
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const int k = kl * KPL + i;
    S[i] = s.pos0 > 0 && live && k < dim ? S0[(size_t)k * a.vdim + col] : 0.f;
    N[i] = s.pos0 > 0 && k < dim ? N0[s.flip * nn + k] : 0.f;
  }
  const int lt = tid >> 4, lk = (tid & 15) * KPL;
  float rq[KPL], rk[KPL], rv = 0.f, ri = 0.f, rf = 0.f;
  const float bi = a.b_i[h], bf = a.b_f[h];
  auto fetch = [&](int t0) {
    const int t = t0 + lt;
    const bool ok = t < s.len;
    const size_t row = (size_t)(s.row0 + (ok ? t : 0));
    const T* P = reinterpret_cast<const T*>(a.proj_t) + row * a.ld;
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      const bool in = ok && lk + i < dim;
      rq[i] = in ? (float)P[a.col_q + h * dim + lk + i] * a.q_scale : 0.f;
      rk[i] = in ? (float)P[a.col_k + h * dim + lk + i] : 0.f;
    }
    const int c = blockIdx.x * 16 + (tid & 15);
    rv = ok && c < a.vdim ? (float)P[a.col_v + h * a.vdim + c] : 0.f;
    const float* G = a.gate_f + row * a.ld_gate;
    ri = a.gate_cap * tanhf((G[a.col_i + h] + bi) / a.gate_cap);
    rf = logsigmoid_f(a.gate_cap * tanhf((G[a.col_f + h] + bf) / a.gate_cap));
  };
  fetch(0);
  for (int t0 = 0; t0 < s.len; t0 += SCAN_CH) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      sq_[lt][lk + i] = rq[i];
      sk_[lt][lk + i] = rk[i];
    }
    sv_[lt][tid & 15] = rv;
    if ((tid & 15) == 0) {
      si_[lt] = ri;
      sf_[lt] = rf;
    }
    __syncthreads();
    if (t0 + SCAN_CH < s.len) fetch(t0 + SCAN_CH);
    const int n = min((int)SCAN_CH, s.len - t0);
    {  // the running maximum of the chunk: thread t of every 16 takes token t, all of them carry the last one on
      float mm = m, keep = 0.f, add = 0.f, fl = 0.f;
      for (int t = 0; t < n; ++t) {
        const float before = mm;
        mm = fmaxf(sf_[t] + mm, si_[t]);
        if (t == (tid & 15)) {
          keep = sf_[t] + before - mm;
          add = si_[t] - mm;
          fl = -mm;
        }
      }
      m = mm;
      if (tid < SCAN_CH) {
        s_keep[tid] = expf(keep);
        s_add[tid] = expf(add);
        s_floor[tid] = expf(fl);
      }
    }
    __syncthreads();
    float q[KPL], k[KPL];  // the current token's; the next one's are read while it is worked off
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      q[i] = sq_[0][kl * KPL + i];
      k[i] = sk_[0][kl * KPL + i];
    }
    float v = sv_[0][vl], keep = s_keep[0], add = s_add[0], fl = s_floor[0];
    for (int t = 0; t < n; ++t) {
      const int t1 = min(t + 1, SCAN_CH - 1);
      float q1[KPL], k1[KPL];
#pragma unroll
      for (int i = 0; i < KPL; ++i) {
        q1[i] = sq_[t1][kl * KPL + i];
        k1[i] = sk_[t1][kl * KPL + i];
      }
      const float v1 = sv_[t1][vl], keep1 = s_keep[t1], add1 = s_add[t1], fl1 = s_floor[t1];
      const float av = add * v;
      float o = 0.f, nq = 0.f;
#pragma unroll
      for (int i = 0; i < KPL; ++i) {
        S[i] = keep * S[i] + av * k[i];
        N[i] = keep * N[i] + add * k[i];
        o += S[i] * q[i];
        nq += N[i] * q[i];
      }
      o = row_sum(o);
      nq = row_sum(nq);
      if (kl == 0 && live) a.o[(size_t)(s.row0 + t0 + t) * nv + (size_t)h * a.vdim + col] = o / (fmaxf(fabsf(nq), fl) + a.floor_eps);
#pragma unroll
      for (int i = 0; i < KPL; ++i) {
        q[i] = q1[i];
        k[i] = k1[i];
      }
      v = v1;
      keep = keep1;
      add = add1;
      fl = fl1;
    }
  }
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const int k = kl * KPL + i;
    if (k < dim && live) S0[(size_t)k * a.vdim + col] = S[i];
    if (k < dim && blockIdx.x == 0 && vl == 0) N0[(s.flip ^ 1) * nn + k] = N[i];
  }
  if (blockIdx.x == 0 && tid == 0) M0[(s.flip ^ 1) * a.heads] = m;
}
template <typename T>
static int mlstm_t(hipStream_t st, const MlstmArgs& a) {
  return by_kpl(a, [&](int kpl) {
    const dim3 grid(cdiv(a.vdim, 16), a.heads, a.p.n_seqs);
    if (kpl == 2) hipLaunchKernelGGL((mlstm_scan_kernel<T, 2>), grid, dim3(256), 0, st, a);
    else if (kpl == 4) hipLaunchKernelGGL((mlstm_scan_kernel<T, 4>), grid, dim3(256), 0, st, a);
    else if (kpl == 8) hipLaunchKernelGGL((mlstm_scan_kernel<T, 8>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((mlstm_scan_kernel<T, 16>), grid, dim3(256), 0, st, a);
    return (int)DSK_OK;
  }, "mlstm");
}
int launch_mlstm_scan(hipStream_t st, const MlstmArgs& a, bool f32) { return f32 ? mlstm_t<float>(st, a) : mlstm_t<bf16>(st, a); }

// ---- wkv: the scan -----------------------------------------------------------------------------------
template <typename T, int KPL>
__global__ __launch_bounds__(256) void wkv_scan_kernel(const WkvArgs a) {
  constexpr int DK = 16 * KPL;
  __shared__ __attribute__((aligned(16))) float sr_[SCAN_CH][DK], sk_[SCAN_CH][DK], sw_[SCAN_CH][DK];
  __shared__ float sv_[SCAN_CH][16], sbonus[SCAN_CH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int kl = lane & 15, vl = wave * 4 + (lane >> 4);
  const int h = blockIdx.y, dim = a.dim, n_all = a.heads * dim;
  const int col = blockIdx.x * 16 + vl;
  const bool live = col < dim;
  const SeqDesc s = a.p.seqs[blockIdx.z];
  float* S0 = reinterpret_cast<float*>(s.state + a.off_s) + (size_t)h * dim * dim;
  float S[KPL];
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const int k = kl * KPL + i;
    S[i] = s.pos0 > 0 && live && k < dim ? S0[(size_t)k * dim + col] : 0.f;
  }
  const int lt = tid >> 4, lk = (tid & 15) * KPL;
  float rr[KPL], rk[KPL], rw[KPL], rv = 0.f, rb = 0.f;
  auto fetch = [&](int t0) {
    const int t = t0 + lt;
    const bool ok = t < s.len;
    const size_t row = (size_t)(s.row0 + (ok ? t : 0));
    const T* P = reinterpret_cast<const T*>(a.proj_t) + row * a.ld + h * dim;
    rb = 0.f;
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      const bool in = ok && lk + i < dim;
      rr[i] = in ? (float)P[a.col_r + lk + i] : 0.f;
      rk[i] = in ? (float)P[a.col_k + lk + i] : 0.f;
      rw[i] = in ? expf(-expf(a.low_f[row * a.ld_low + h * dim + lk + i] + a.w0[h * dim + lk + i])) : 0.f;
      rb += in ? rr[i] * a.u[h * dim + lk + i] * rk[i] : 0.f;
    }
    rb = row_sum(rb);
    const int c = blockIdx.x * 16 + (tid & 15);
    rv = ok && c < dim ? (float)P[a.col_v + c] : 0.f;
  };
  fetch(0);
  for (int t0 = 0; t0 < s.len; t0 += SCAN_CH) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      sr_[lt][lk + i] = rr[i];
      sk_[lt][lk + i] = rk[i];
      sw_[lt][lk + i] = rw[i];
    }
    sv_[lt][tid & 15] = rv;
    if ((tid & 15) == 0) sbonus[lt] = rb;
    __syncthreads();
    if (t0 + SCAN_CH < s.len) fetch(t0 + SCAN_CH);
    const int n = min((int)SCAN_CH, s.len - t0);
    for (int t = 0; t < n; ++t) {
      const float v = sv_[t][vl];
      float o = 0.f;
#pragma unroll
      for (int i = 0; i < KPL; ++i) {
        o += S[i] * sr_[t][kl * KPL + i];
        S[i] = sw_[t][kl * KPL + i] * S[i] + sk_[t][kl * KPL + i] * v;
      }
      o = row_sum(o);
      if (kl == 0 && live) a.o[(size_t)(s.row0 + t0 + t) * n_all + h * dim + col] = o + sbonus[t] * v;
    }
  }
  if (live)
#pragma unroll
    for (int i = 0; i < KPL; ++i) {
      const int k = kl * KPL + i;
      if (k < dim) S0[(size_t)k * dim + col] = S[i];
    }
}
template <typename T>
static int wkv_t(hipStream_t st, const WkvArgs& a) {
  return by_kpl(a, [&](int kpl) {
    const dim3 grid(cdiv(a.dim, 16), a.heads, a.p.n_seqs);
    if (kpl == 2) hipLaunchKernelGGL((wkv_scan_kernel<T, 2>), grid, dim3(256), 0, st, a);
    else if (kpl == 4) hipLaunchKernelGGL((wkv_scan_kernel<T, 4>), grid, dim3(256), 0, st, a);
    else if (kpl == 8) hipLaunchKernelGGL((wkv_scan_kernel<T, 8>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((wkv_scan_kernel<T, 16>), grid, dim3(256), 0, st, a);
    return (int)DSK_OK;
  }, "wkv");
}
int launch_wkv_scan(hipStream_t st, const WkvArgs& a, bool f32) { return f32 ? wkv_t<float>(st, a) : wkv_t<bf16>(st, a); }
template <typename T>
__global__ __launch_bounds__(256) void wkv_out_kernel(const WkvArgs a) {
  const size_t row = blockIdx.x;
  const float* o = a.o + row * a.heads * a.dim;
  const T* gp = reinterpret_cast<const T*>(a.proj_t) + row * a.ld + a.col_g;
  head_norm_gate<T>([&](int h, int i) { return o[h * a.dim + i]; }, a.heads, a.dim, a.eps, a.out_norm, false, [&](int c) { return silu_f((float)gp[c]); },
                    reinterpret_cast<T*>(a.out_t) + row * a.out_ld);
}
int launch_wkv_out(hipStream_t st, const WkvArgs& a, bool f32) {
  if (f32) hipLaunchKernelGGL(wkv_out_kernel<float>, dim3(a.p.rows), dim3(256), 0, st, a);
  else hipLaunchKernelGGL(wkv_out_kernel<bf16>, dim3(a.p.rows), dim3(256), 0, st, a);
  return DSK_OK;
}
