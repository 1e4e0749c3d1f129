// Gated delta rule: one fp32 state matrix S [key][value] per (sequence, head) kept in a state slot between steps, with
// one decay per head and key channel and q / k / v behind a short causal convolution (short_conv.h):
//   q, k, v <- silu(conv(.));  q <- q / sqrt(sum q^2 + unit_eps) * q_scale;  k <- k / sqrt(sum k^2 + unit_eps)
//   g = exp(-decay[h] softplus(z));  beta = sigmoid(b)
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//   out = o / rms(o) * nw * sigmoid(gate)                               (rms over the head's value channels)
// Query / key heads may be fewer than value heads (head h reads q / k head h / (H / G)). Three launches:
//   prep   (token, q / k head) parallel: convolutions, unit norms, decays; per (head, channel) the fp32 vector
//          {g, beta k, q, g k} (with it the update is S <- g S + (beta k)(v - (g k)^T S_old)) and the values.
//   scan   the recurrence. Column v of S depends on no other column: a wave owns CL NC columns of one head, lane =
//          (key group of KG, column group of CL = 64 / KG), lane q of a column holding the keys q, q + KG, ...: DQ
//          state entries per column in registers, the two sums over keys are DQ FMAs and log2(KG) lane exchanges. A
//          workgroup's four waves share the tokens' vectors, staged through LDS TC tokens at a time while the next
//          TC are loaded into registers. KG 32 with one column per lane: the shortest chain per token, for few
//          sequences; KG 8 with four adjacent columns per lane: least work and whole cache lines of the state, for
//          many. A sequence's tokens of the step run in order from the slot's state; a portion that starts at
//          position 0 starts from zero, so a reused slot needs no clearing.
//   finish (token, four heads) parallel: head RMS norm, norm weight, output gate, store; the blocks of a portion's last
//          token also rewrite the slot's kept convolution inputs.
// Long steps (a prompt portion of hundreds of tokens; D <= 128, V <= 256, at most four taps) take chunks of CN = 32 tokens at once. With S the
// state a chunk starts from, gamma_i = g_1 .. g_i per channel and
//   a_ij = sum_d k_i k_j g_(j+1) .. g_i (j < i),   b_ij = sum_d q_i k_j g_(j+1) .. g_i (j <= i)
// the tokens' updates solve a unit lower triangular system that does not involve S:
//   w_i = beta_i (gamma_i k_i - sum_(j<i) a_ij w_j),   v'_i = beta_i (v_i - sum_(j<i) a_ij v'_j),   u_i = v'_i - S^T w_i
//   o_i = S^T (gamma_i q_i - sum_(j<=i) b_ij w_j) + sum_(j<=i) b_ij v'_j
//   S  <- diag(gamma_CN) S + sum_j (g_(j+1) .. g_CN k_j) u_j^T
// Every product of decays is a product of factors <= 1 taken in order (nothing is divided by a decay). Three launches:
//   chunk  (chunk, head) parallel: convolutions, norms, decays (LDS), a and b (a lane holds k_j g_(j+1) .. g_i of four D / 32
//          channels and walks i), the triangular solve with one column of [w | v'] per thread, all fp32.
//   chunk scan    the only sequential part: per (sequence, head, 16 columns) S^T [w; q'] and the update as fp32 MFMA
//          (16x16x4) over the chunks; S stays in registers (C layout) and goes round through LDS as B operand.
//   chunk finish  as finish, from the scan's [column][token] tiles.
// Rows past a portion's end are tokens with k = q = v = 0, g = 1, beta = 0.
#include "common.h"
#include "seq_launchers.h"
#include "short_conv.h"

namespace vgate {
namespace {

__device__ __forceinline__ float sigm(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float silu_f(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
template <int CTRL>
__device__ __forceinline__ float row_rot(float v) {  // a rotation inside each row of 16 lanes (DPP), on the VALU
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false));
}
// sum over the KG lanes that share lane % (64 / KG)
template <int KG>
__device__ __forceinline__ float key_sum(float v) {
  if (KG >= 32) v += row_rot<0x122>(v);   // lanes 2 apart
  if (KG >= 16) v += row_rot<0x124>(v);   // 4
  v += row_rot<0x128>(v);                 // 8
  v += xor16(v);
  v += xor32(v);
  return v;
}

// grid (token, q / k head)
__global__ __launch_bounds__(256) void gated_delta_prep_kernel(GatedDeltaArgs p, float4* __restrict__ vec,
                                                                float* __restrict__ vals) {
  extern __shared__ float qk[];  // q [D], then k [D]
  __shared__ float inv[2];
  const int t = blockIdx.x, g = blockIdx.y;
  if (t >= p.query_start[p.S]) return;  // padding rows of a graph bucket
  const int s = seq_of_row(p.query_start, p.S, t);
  const int slot = p.state_slots[s];
  if (slot < 0) return;
  const int t0 = p.query_start[s], pos0 = p.context_lens[s] - (p.query_start[s + 1] - t0);
  const int D = p.D, V = p.V, GD = p.G * D, HV = p.H * V, rep = p.H / p.G, NC = 2 * GD + HV;
  const float* kept = p.conv_state + (int64_t)slot * (p.taps - 1) * NC;
  const int tid = threadIdx.x;
  for (int e = tid; e < 2 * D; e += 256) {
    const bool isq = e < D;
    const int c = g * D + (isq ? e : e - D), col = isq ? c : GD + c;
    qk[e] = silu_f(short_conv_at(isq ? p.q : p.k, isq ? p.ldq : p.ldk, p.f32, c, p.conv_w, NC, col, 0.f, kept, NC, col, t, t0,
                                 pos0, p.taps));
  }
  for (int e = tid; e < rep * V; e += 256) {
    const int c = g * rep * V + e, col = 2 * GD + c;
    vals[(int64_t)t * HV + c] = silu_f(short_conv_at(p.v, p.ldv, p.f32, c, p.conv_w, NC, col, 0.f, kept, NC, col, t, t0, pos0, p.taps));
  }
  __syncthreads();
  if (tid < 128) {  // wave 0: q, wave 1: k
    const float* x = qk + (tid >> 6) * D;
    float ss = 0.f;
    for (int d = tid & 63; d < D; d += 64) ss = fmaf(x[d], x[d], ss);
    ss = wave_reduce_sum(ss);
    if ((tid & 63) == 0) inv[tid >> 6] = 1.f / sqrtf(ss + p.unit_eps);
  }
  __syncthreads();
  const float qi = inv[0] * p.q_scale, ki = inv[1];
  for (int e = tid; e < rep * D; e += 256) {
    const int h = g * rep + e / D, d = e % D;
    const float z = p.z[(int64_t)t * p.ldz + h * D + d];
    const float a = expf(-p.decay[h] * softplus_f(z));
    const float beta = sigm(conv_ldx(p.b, (int64_t)t * p.ldb + h, p.f32));
    const float k = qk[D + d] * ki;
    vec[((int64_t)t * p.H + h) * D + d] = make_float4(a, beta * k, qk[d] * qi, a * k);
  }
}

// grid (sequence, head, column slice of 4 CW)
template <int KG, int NC, int DQ, int TC>
__global__ __launch_bounds__(256) void gated_delta_scan_kernel(GatedDeltaArgs p, const float4* __restrict__ vec,
                                                                const float* __restrict__ vals, float* __restrict__ oraw) {
  constexpr int CL = 64 / KG, CW = CL * NC, DP = KG * DQ;
  constexpr int NV = (TC * DP + 255) / 256, NVL = (TC * 4 * CW + 255) / 256;
  __shared__ __attribute__((aligned(16))) float4 lv[2][TC][DP];
  __shared__ __attribute__((aligned(16))) float lvv[2][TC][4 * CW];
  const int s = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * 4 * CW;
  const int slot = p.state_slots[s];
  const int t0 = p.query_start[s], t1 = p.query_start[s + 1];
  if (slot < 0 || t1 <= t0) return;
  const int D = p.D, V = p.V, H = p.H;
  const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, q = lane / CL, cl = lane % CL;
  const int c = c0 + wv * CW + cl * NC;   // the lane's first column
  const bool from_zero = p.context_lens[s] - (t1 - t0) <= 0;
  float* sp = p.state + ((int64_t)slot * H + h) * D * V;
  float S[DQ][NC];
#pragma unroll
  for (int j = 0; j < DQ; ++j)
#pragma unroll
    for (int n = 0; n < NC; ++n)
      S[j][n] = (!from_zero && j * KG + q < D && c + n < V) ? sp[(int64_t)(j * KG + q) * V + c + n] : 0.f;
  float4 pv[NV];
  float pvv[NVL];
  auto fetch = [&](int tb) {
#pragma unroll
    for (int r = 0; r < NV; ++r) {
      const int e = tid + 256 * r, i = e / DP, d = e % DP;
      pv[r] = (e < TC * DP && d < D && tb + i < t1) ? vec[((int64_t)(tb + i) * H + h) * D + d] : make_float4(0.f, 0.f, 0.f, 0.f);
    }
#pragma unroll
    for (int r = 0; r < NVL; ++r) {
      const int e = tid + 256 * r, i = e / (4 * CW), cc = c0 + e % (4 * CW);
      pvv[r] = (e < TC * 4 * CW && cc < V && tb + i < t1) ? vals[((int64_t)(tb + i) * H + h) * V + cc] : 0.f;
    }
  };
  auto put = [&](int buf) {  // (channels past D are zero vectors: they leave S and both sums alone)
#pragma unroll
    for (int r = 0; r < NV; ++r) {
      const int e = tid + 256 * r;
      if (e < TC * DP) (&lv[buf][0][0])[e] = pv[r];
    }
#pragma unroll
    for (int r = 0; r < NVL; ++r) {
      const int e = tid + 256 * r;
      if (e < TC * 4 * CW) (&lvv[buf][0][0])[e] = pvv[r];
    }
  };
  fetch(t0);
  put(0);
  __syncthreads();
  int buf = 0;
  for (int tb = t0; tb < t1; tb += TC) {
    const bool more = tb + TC < t1;
    if (more) fetch(tb + TC);
    const int nt = min(TC, t1 - tb);
    // token i + 1's vectors are read from LDS before token i's sums and lane exchanges (they do not depend on the state)
    float4 x[2][DQ];
    float vv[2][NC];
    auto grab = [&](int i, int r) {
#pragma unroll
      for (int j = 0; j < DQ; ++j) x[r][j] = lv[buf][i][j * KG + q];
#pragma unroll
      for (int n = 0; n < NC; ++n) vv[r][n] = lvv[buf][i][wv * CW + cl * NC + n];
    };
    grab(0, 0);
#pragma unroll
    for (int i = 0; i < TC; ++i) {
      if (i >= nt) break;
      if (i + 1 < TC) grab(i + 1, (i + 1) & 1);  // (past nt: zero vectors, never used)
      const int r = i & 1;
      float u[NC], o[NC];
#pragma unroll
      for (int n = 0; n < NC; ++n) {
        u[n] = 0.f; o[n] = 0.f;
      }
#pragma unroll
      for (int j = 0; j < DQ; ++j)
#pragma unroll
        for (int n = 0; n < NC; ++n) u[n] = fmaf(x[r][j].w, S[j][n], u[n]);
#pragma unroll
      for (int n = 0; n < NC; ++n) u[n] = vv[r][n] - key_sum<KG>(u[n]);
#pragma unroll
      for (int j = 0; j < DQ; ++j)
#pragma unroll
        for (int n = 0; n < NC; ++n) {
          S[j][n] = fmaf(x[r][j].y, u[n], x[r][j].x * S[j][n]);
          o[n] = fmaf(x[r][j].z, S[j][n], o[n]);
        }
#pragma unroll
      for (int n = 0; n < NC; ++n) {
        o[n] = key_sum<KG>(o[n]);
        if (q == 0 && c + n < V) oraw[((int64_t)(tb + i) * H + h) * V + c + n] = o[n];
      }
    }
    if (more) {
      put(buf ^ 1);   // (the other buffer: every wave left it at the barrier before this tile)
      __syncthreads();
      buf ^= 1;
    }
  }
#pragma unroll
  for (int j = 0; j < DQ; ++j)
#pragma unroll
    for (int n = 0; n < NC; ++n)
      if (j * KG + q < D && c + n < V) sp[(int64_t)(j * KG + q) * V + c + n] = S[j][n];
}

// grid (token, stretch of four heads): one head per wave
__global__ __launch_bounds__(256) void gated_delta_finish_kernel(GatedDeltaArgs p, const float* __restrict__ oraw) {
  const int t = blockIdx.x;
  if (t >= p.query_start[p.S]) return;
  const int H = p.H, V = p.V, D = p.D, GD = p.G * D, HV = H * V;
  const int s = seq_of_row(p.query_start, p.S, t);
  const int slot = p.state_slots[s];
  if (slot < 0) return;
  const int wv = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const float* o = oraw + (int64_t)t * HV;
  for (int h = 4 * blockIdx.y + wv; h < H; h += 4 * gridDim.y) {
    float ss = 0.f;
    for (int c = lane; c < V; c += 64) ss = fmaf(o[h * V + c], o[h * V + c], ss);
    ss = wave_reduce_sum(ss);
    const float rn = 1.f / sqrtf(ss / (float)V + p.eps);
    for (int c = lane; c < V; c += 64) {
      const float y = o[h * V + c] * rn * p.nw[c] * sigm(p.gate[(int64_t)t * p.ldg + h * V + c]);
      const int64_t oi = (int64_t)t * p.ldo + h * V + c;
      if (p.f32) reinterpret_cast<float*>(p.out)[oi] = y;
      else reinterpret_cast<bf16_t*>(p.out)[oi] = f2bf(y);
    }
  }
  const int t0 = p.query_start[s], t1 = p.query_start[s + 1];
  if (t != t1 - 1 || p.taps < 2) return;
  const int pos0 = p.context_lens[s] - (t1 - t0), NC = 2 * GD + HV;
  float* kept = p.conv_state + (int64_t)slot * (p.taps - 1) * NC;
  for (int e = blockIdx.y * 256 + threadIdx.x; e < NC; e += 256 * gridDim.y) {
    const void* x = e < GD ? p.q : (e < 2 * GD ? p.k : p.v);
    const int64_t ld = e < GD ? p.ldq : (e < 2 * GD ? p.ldk : p.ldv);
    short_conv_keep(x, ld, p.f32, e < GD ? e : (e < 2 * GD ? e - GD : e - 2 * GD), kept, NC, e, t0, t1, pos0, p.taps);
  }
}

// ------------------------------------------------------------------------------------------ chunks of CN tokens
constexpr int CN = 32;
// floats of one (chunk, head) record: [w; q'] [2 CN][DP], the update's keys [DP][CN], gamma_CN [DP], v' [V][CN], and b v', which
// becomes o [V][CN]
__host__ __device__ inline int64_t chunk_floats(int DP, int V) { return (int64_t)3 * CN * DP + DP + (int64_t)2 * CN * V; }

__device__ __forceinline__ bool locate_chunk(const GatedDeltaArgs& p, int bx, int& s, int& t0, int& t1) {
  int base = 0;
  for (int i = 0; i < p.S; ++i) {
    const int a = p.query_start[i], b = p.query_start[i + 1];
    const int nc = (p.state_slots[i] < 0 || b <= a) ? 0 : (b - a + CN - 1) / CN;
    if (bx < base + nc) {
      s = i; t0 = a + (bx - base) * CN; t1 = min(b, t0 + CN);
      return true;
    }
    base += nc;
  }
  return false;
}

// sum over j < n (a constant after unrolling) of row[j] x[j]; the row is read in 16-B pieces
__device__ __forceinline__ float row_dot(const float* row, const float (&x)[CN], int n) {
  float a = 0.f, b = 0.f;   // (two chains)
#pragma unroll
  for (int j0 = 0; j0 < CN; j0 += 4)
    if (j0 < n) {
      const float4 v = *reinterpret_cast<const float4*>(row + j0);
      a = fmaf(v.x, x[j0], a);
      if (j0 + 1 < n) b = fmaf(v.y, x[j0 + 1], b);
      if (j0 + 2 < n) a = fmaf(v.z, x[j0 + 2], a);
      if (j0 + 3 < n) b = fmaf(v.w, x[j0 + 3], b);
    }
  return a + b;
}

// first float of row i of a packed lower triangle whose row i has i entries, padded to whole 16-B pieces (row i of one with
// the diagonal: tri(i + 1))
__host__ __device__ constexpr int tri(int i) {
  const int n = i > 0 ? i - 1 : 0, g = n / 4;
  return i > 0 ? 4 * (2 * g * (g + 1) + (n - 4 * g) * (g + 1)) : 0;
}

// grid (chunk, head). At DP = 128 the LDS comes to a third of a CU's.
template <int DP, bool F32>
__global__ __launch_bounds__(256, DP > 64 ? 3 : 4) void gated_delta_chunk_kernel(GatedDeltaArgs p, float* __restrict__ rec) {
  constexpr int X = DP / 32;   // 16-B pieces of a row a lane of the pair sums holds: channels 32 x + 4 dg ..
  __shared__ __attribute__((aligned(16))) float lk[CN][DP], lq[CN][DP], lg[CN][DP];
  __shared__ __attribute__((aligned(16))) float As[tri(CN)], Bs[tri(CN + 1)];
  __shared__ float beta[CN];
  int s, t0, t1;
  if (!locate_chunk(p, blockIdx.x, s, t0, t1)) return;
  const int h = blockIdx.y, D = p.D, V = p.V, H = p.H, GD = p.G * D;
  const int NC = 2 * GD + H * V, g = h / (H / p.G);
  const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63;
  const int ts = p.query_start[s], te = p.query_start[s + 1], pos0 = p.context_lens[s] - (te - ts);
  const float* kept = p.conv_state + (int64_t)p.state_slots[s] * (p.taps - 1) * NC;
  float* r0 = rec + ((int64_t)blockIdx.x * H + h) * chunk_floats(DP, V);
  float* kt = r0 + 2 * CN * DP;
  float* gam = kt + CN * DP;
  float* vh = gam + DP;
  float* cc = vh + CN * V;
  for (int e = tid; e < 2 * DP; e += 256) {
    const bool isq = e < DP;
    const int d = isq ? e : e - DP, c = g * D + d, col = isq ? c : GD + c;
#pragma unroll 2
    for (int i0 = 0; i0 < CN; i0 += 8) {
      float y[8];
      if (d < D) short_conv_run8<F32>(isq ? p.q : p.k, isq ? p.ldq : p.ldk, c, p.conv_w, NC, col, kept, NC, col, t0 + i0, ts, te, pos0,
                                      p.taps, y);
#pragma unroll
      for (int u = 0; u < 8; ++u) (isq ? lq : lk)[i0 + u][d] = (d < D && t0 + i0 + u < t1) ? silu_f(y[u]) : 0.f;
    }
  }
  const float dec = p.decay[h];
  for (int e = tid; e < CN * DP; e += 256) {
    const int i = e / DP, d = e % DP;
    lg[i][d] = (d < D && t0 + i < t1) ? expf(-dec * softplus_f(p.z[(int64_t)(t0 + i) * p.ldz + h * D + d])) : 1.f;
  }
  if (tid < CN) beta[tid] = t0 + tid < t1 ? sigm(conv_ldx(p.b, (int64_t)(t0 + tid) * p.ldb + h, F32 ? 1 : 0)) : 0.f;
  __syncthreads();
  {  // unit norms of q (times q_scale) and k in place: four threads per row
    const int row = tid >> 2, part = tid & 3;
    float* x = row < CN ? lq[row] : lk[row - CN];
    float4 v[DP / 16];
    float ss = 0.f;
#pragma unroll
    for (int m = 0; m < DP / 16; ++m) {
      v[m] = *reinterpret_cast<const float4*>(x + 16 * m + 4 * part);
      ss = fmaf(v[m].x, v[m].x, fmaf(v[m].y, v[m].y, fmaf(v[m].z, v[m].z, fmaf(v[m].w, v[m].w, ss))));
    }
    ss += row_rot<0xB1>(ss);   // (quad_perm [1, 0, 3, 2], then [2, 3, 0, 1])
    ss += row_rot<0x4E>(ss);
    const float f = 1.f / sqrtf(ss + p.unit_eps) * (row < CN ? p.q_scale : 1.f);
#pragma unroll
    for (int m = 0; m < DP / 16; ++m)
      *reinterpret_cast<float4*>(x + 16 * m + 4 * part) = make_float4(v[m].x * f, v[m].y * f, v[m].z * f, v[m].w * f);
  }
  __syncthreads();
  {  // a and b: a wave owns eight columns j, lane = (channel group dg of eight, j); the wave with most rows differs
     // between neighbouring chunks, so that workgroups on one CU do not all load the same SIMD
    const int jb = (blockIdx.x & 1) ? 3 - wv : wv;
    const int dg = lane >> 3, j = 8 * jb + (lane & 7);
    float r[4 * X];
#pragma unroll
    for (int x = 0; x < X; ++x) {
      const float4 v = *reinterpret_cast<const float4*>(&lk[j][32 * x + 4 * dg]);
      r[4 * x] = v.x; r[4 * x + 1] = v.y; r[4 * x + 2] = v.z; r[4 * x + 3] = v.w;
    }
    for (int i = 8 * jb; i < CN; ++i) {
      float a = 0.f, b = 0.f;
#pragma unroll
      for (int x = 0; x < X; ++x) {
        const float4 gv = *reinterpret_cast<const float4*>(&lg[i][32 * x + 4 * dg]);
        const float4 kv = *reinterpret_cast<const float4*>(&lk[i][32 * x + 4 * dg]);
        const float4 qv = *reinterpret_cast<const float4*>(&lq[i][32 * x + 4 * dg]);
        if (i > j) { r[4 * x] *= gv.x; r[4 * x + 1] *= gv.y; r[4 * x + 2] *= gv.z; r[4 * x + 3] *= gv.w; }
        a = fmaf(r[4 * x], kv.x, fmaf(r[4 * x + 1], kv.y, fmaf(r[4 * x + 2], kv.z, fmaf(r[4 * x + 3], kv.w, a))));
        b = fmaf(r[4 * x], qv.x, fmaf(r[4 * x + 1], qv.y, fmaf(r[4 * x + 2], qv.z, fmaf(r[4 * x + 3], qv.w, b))));
      }
      a = key_sum<8>(a);
      b = key_sum<8>(b);
      if (dg == 0 && i > j) As[tri(i) + j] = a;
      if (dg == 0 && i >= j) Bs[tri(i + 1) + j] = b;
    }
  }
  __syncthreads();
  for (int c = tid; c < D + V; c += 256) {   // one column of [w | v'] per thread
    float x[CN];
    if (c < D) {
      float gm = 1.f;
#pragma unroll
      for (int i = 0; i < CN; ++i) {
        gm *= lg[i][c];
        x[i] = gm * lk[i][c];
      }
    } else {
      const int vc = h * V + c - D, col = 2 * GD + vc;
#pragma unroll
      for (int i0 = 0; i0 < CN; i0 += 8) {
        float y[8];
        short_conv_run8<F32>(p.v, p.ldv, vc, p.conv_w, NC, col, kept, NC, col, t0 + i0, ts, te, pos0, p.taps, y);
#pragma unroll
        for (int u = 0; u < 8; ++u) x[i0 + u] = t0 + i0 + u < t1 ? silu_f(y[u]) : 0.f;
      }
    }
#pragma unroll
    for (int i = 0; i < CN; ++i) {
      x[i] = beta[i] * (x[i] - row_dot(As + tri(i), x, i));
      if (i % 2) __builtin_amdgcn_sched_barrier(0);   // (rows ahead of time would take hundreds of registers)
    }
    if (c < D) {
      float gb = 1.f;
#pragma unroll
      for (int j0 = CN - 4; j0 >= 0; j0 -= 4) {
        f32x4 v;
#pragma unroll
        for (int j = 3; j >= 0; --j) {
          v[j] = lk[j0 + j][c] * gb;
          gb *= lg[j0 + j][c];
        }
        *reinterpret_cast<f32x4*>(kt + c * CN + j0) = v;
        __builtin_amdgcn_sched_barrier(0);
      }
      gam[c] = gb;
      float gm = 1.f;
#pragma unroll
      for (int i = 0; i < CN; ++i) {
        gm *= lg[i][c];
        r0[i * DP + c] = x[i];
        r0[(CN + i) * DP + c] = gm * lq[i][c] - row_dot(Bs + tri(i + 1), x, i + 1);
        if (i % 2) __builtin_amdgcn_sched_barrier(0);
      }
    } else {
#pragma unroll
      for (int i0 = 0; i0 < CN; i0 += 4) {
        f32x4 v;
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = row_dot(Bs + tri(i0 + i + 1), x, i0 + i + 1);
        *reinterpret_cast<f32x4*>(vh + (c - D) * CN + i0) = f32x4{x[i0], x[i0 + 1], x[i0 + 2], x[i0 + 3]};
        *reinterpret_cast<f32x4*>(cc + (c - D) * CN + i0) = v;
        __builtin_amdgcn_sched_barrier(0);
      }
    }
  }
  for (int e = tid; e < (DP - D) * CN; e += 256) {   // channels past D: zero
    const int d = D + e / CN, i = e % CN;
    r0[i * DP + d] = 0.f;
    r0[(CN + i) * DP + d] = 0.f;
    kt[d * CN + i] = 0.f;
    if (i == 0) gam[d] = 0.f;
  }
}

__device__ __forceinline__ f32x4 ld4(const float* p) {
  const float4 v = *reinterpret_cast<const float4*>(p);
  return f32x4{v.x, v.y, v.z, v.w};
}

// grid (head, rounded up to the XCDs, 16 columns, sequence): a head's workgroups read the same records on one XCD. NT tiles
// of 16 channels. MFMA operands: the channel (or token) 16 n + 4 kg + e is element e of lane group kg in both operands, so
// a lane's four steps are one 16-B piece of a row.
template <int NT>
__global__ __launch_bounds__(256) void gated_delta_chunk_scan_kernel(GatedDeltaArgs p, float* __restrict__ rec) {
  constexpr int DP = 16 * NT, TW = (NT + 3) / 4;
  __shared__ __attribute__((aligned(16))) float Sl[16][DP + 4];
  __shared__ __attribute__((aligned(16))) float Ul[16][CN + 4];
  const int s = blockIdx.z, h = blockIdx.x, c0 = blockIdx.y * 16;
  if (h >= p.H) return;
  const int slot = p.state_slots[s];
  const int t0 = p.query_start[s], t1 = p.query_start[s + 1];
  if (slot < 0 || t1 <= t0) return;
  int base = 0;
  for (int i = 0; i < s; ++i) {
    const int a = p.query_start[i], b = p.query_start[i + 1];
    base += (p.state_slots[i] < 0 || b <= a) ? 0 : (b - a + CN - 1) / CN;
  }
  const int nc = (t1 - t0 + CN - 1) / CN, D = p.D, V = p.V, H = p.H;
  const int w = threadIdx.x >> 6, l = threadIdx.x & 63, lr = l & 15, kg = l >> 4;
  const bool con = c0 + lr < V;
  const int col = con ? c0 + lr : V - 1;   // (a column past the last: computed on the last one's inputs, never stored)
  const bool from_zero = p.context_lens[s] - (t1 - t0) <= 0;
  float* sp = p.state + ((int64_t)slot * H + h) * D * V;
  f32x4 S[TW];
#pragma unroll
  for (int t = 0; t < TW; ++t) {
    const int tile = w + 4 * t;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * tile + 4 * kg + i;
      S[t][i] = (!from_zero && tile < NT && d < D && con) ? sp[(int64_t)d * V + c0 + lr] : 0.f;
    }
    if (tile < NT) *reinterpret_cast<f32x4*>(&Sl[lr][16 * tile + 4 * kg]) = S[t];
  }
  const int64_t per = chunk_floats(DP, V);
  float* r0 = rec + ((int64_t)base * H + h) * per;
  struct Chunk {   // what a lane needs of one chunk's record
    f32x4 A[NT], K[TW][2], gm[TW], add;
    float* vc;
  };
  auto fetch = [&](Chunk& x, int ch) {
    float* r = r0 + (int64_t)ch * H * per;
    const float* kt = r + 2 * CN * DP;
    float* gam = r + 3 * CN * DP;
    x.vc = gam + DP + (w < 2 ? 0 : CN * V) + (int64_t)col * CN + 16 * (w & 1) + 4 * kg;   // v' of waves 0, 1; b v' / o of 2, 3
#pragma unroll
    for (int n = 0; n < NT; ++n) x.A[n] = ld4(r + (16 * w + lr) * DP + 16 * n + 4 * kg);
    x.add = ld4(x.vc);
#pragma unroll
    for (int t = 0; t < TW; ++t) {
      const int tile = min(w + 4 * t, NT - 1);
      x.gm[t] = ld4(gam + 16 * tile + 4 * kg);
      x.K[t][0] = ld4(kt + (16 * tile + lr) * CN + 4 * kg);
      x.K[t][1] = ld4(kt + (16 * tile + lr) * CN + 16 + 4 * kg);
    }
  };
  // chunk ch from `x`, while chunk ch + 1 is on its way into `y` (the barriers wait for LDS traffic only)
  auto step = [&](Chunk& x, Chunk& y, int ch) {
    fetch(y, min(ch + 1, nc - 1));   // (without a branch: the waits below then count past these loads)
    __builtin_amdgcn_sched_barrier(0);
    f32x4 P0 = f32x4{0.f, 0.f, 0.f, 0.f}, P1 = P0;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
      const f32x4 b = *reinterpret_cast<const f32x4*>(&Sl[lr][16 * n + 4 * kg]);
      P0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.A[n][0], b[0], P0, 0, 0, 0);
      P1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.A[n][1], b[1], P1, 0, 0, 0);
      P0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.A[n][2], b[2], P0, 0, 0, 0);
      P1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.A[n][3], b[3], P1, 0, 0, 0);
    }
    const f32x4 P = P0 + P1;
    if (w < 2) *reinterpret_cast<f32x4*>(&Ul[lr][16 * w + 4 * kg]) = x.add - P;
    else if (con) *reinterpret_cast<f32x4*>(x.vc) = x.add + P;
    lds_barrier();   // u is there, and every wave is done with S
#pragma unroll
    for (int t = 0; t < TW; ++t) {
      S[t] *= x.gm[t];
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        const f32x4 b = *reinterpret_cast<const f32x4*>(&Ul[lr][16 * m + 4 * kg]);
#pragma unroll
        for (int e = 0; e < 4; ++e) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.K[t][m][e], b[e], S[t], 0, 0, 0);
      }
      if (w + 4 * t < NT) *reinterpret_cast<f32x4*>(&Sl[lr][16 * (w + 4 * t) + 4 * kg]) = S[t];
    }
    lds_barrier();
  };
  Chunk x, y;
  fetch(x, 0);
  lds_barrier();
  int ch = 0;
  for (; ch + 1 < nc; ch += 2) {
    step(x, y, ch);
    step(y, x, ch + 1);
  }
  if (ch < nc) step(x, y, ch);
#pragma unroll
  for (int t = 0; t < TW; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * (w + 4 * t) + 4 * kg + i;
      if (w + 4 * t < NT && d < D && con) sp[(int64_t)d * V + c0 + lr] = S[t][i];
    }
}

constexpr int CHUNK_MAX_V = 256;
// grid (chunk, head)
__global__ __launch_bounds__(256) void gated_delta_chunk_finish_kernel(GatedDeltaArgs p, int DP, const float* __restrict__ rec) {
  __shared__ float lo[CHUNK_MAX_V][CN + 1];
  __shared__ float rn[CN];
  int s, t0, t1;
  if (!locate_chunk(p, blockIdx.x, s, t0, t1)) return;
  const int h = blockIdx.y, V = p.V, H = p.H, tid = threadIdx.x;
  const float* o = rec + ((int64_t)blockIdx.x * H + h) * chunk_floats(DP, V) + 3 * CN * DP + DP + CN * V;
  for (int e = tid; e < V * CN; e += 256) lo[e / CN][e % CN] = o[e];
  __syncthreads();
  {  // eight threads per token
    const int i = tid >> 3, part = tid & 7;
    float ss = 0.f;
    for (int c = part; c < V; c += 8) ss = fmaf(lo[c][i], lo[c][i], ss);
    ss += row_rot<0xB1>(ss);
    ss += row_rot<0x4E>(ss);
    ss += row_rot<0x141>(ss);   // (row_half_mirror: the other four of the eight)
    if (part == 0) rn[i] = 1.f / sqrtf(ss / (float)V + p.eps);
  }
  __syncthreads();
  for (int e = tid; e < (t1 - t0) * V; e += 256) {
    const int i = e / V, c = e % V;
    const int64_t t = t0 + i;
    const float y = lo[c][i] * rn[i] * p.nw[c] * sigm(p.gate[t * p.ldg + h * V + c]);
    const int64_t oi = t * p.ldo + h * V + c;
    if (p.f32) reinterpret_cast<float*>(p.out)[oi] = y;
    else reinterpret_cast<bf16_t*>(p.out)[oi] = f2bf(y);
  }
  const int ts = p.query_start[s], te = p.query_start[s + 1];
  if (t1 != te || p.taps < 2) return;
  // the portion's last chunk: this head's value channels and, for the first head of its group, the group's q / k channels
  const int D = p.D, GD = p.G * D, NC = 2 * GD + H * V, rep = H / p.G, pos0 = p.context_lens[s] - (te - ts);
  float* kept = p.conv_state + (int64_t)p.state_slots[s] * (p.taps - 1) * NC;
  const int nq = h % rep == 0 ? 2 * D : 0;
  for (int e = tid; e < nq + V; e += 256) {
    if (e < nq) {
      const bool isq = e < D;
      const int c = (h / rep) * D + (isq ? e : e - D), kc = isq ? c : GD + c;
      short_conv_keep(isq ? p.q : p.k, isq ? p.ldq : p.ldk, p.f32, c, kept, NC, kc, ts, te, pos0, p.taps);
    } else {
      const int c = h * V + e - nq;
      short_conv_keep(p.v, p.ldv, p.f32, c, kept, NC, 2 * GD + c, ts, te, pos0, p.taps);
    }
  }
}

int chunk_channels(int D) { return D <= 32 ? 32 : (D <= 64 ? 64 : 128); }
bool takes_chunks(int T, int S, int D, int V) { return T >= 128 && T >= 64 * S && D <= 128 && V <= CHUNK_MAX_V; }
constexpr int CHUNK_MAX_TAPS = 4;

template <int DP>
void launch_chunks(const GatedDeltaArgs& a, int T, float* rec, hipStream_t st) {
  const int chunks = T / CN + a.S;
  const int hx = (a.H + 7) / 8 * 8;
  if (a.f32) hipLaunchKernelGGL((gated_delta_chunk_kernel<DP, true>), dim3(chunks, a.H), dim3(256), 0, st, a, rec);
  else hipLaunchKernelGGL((gated_delta_chunk_kernel<DP, false>), dim3(chunks, a.H), dim3(256), 0, st, a, rec);
  hipLaunchKernelGGL(gated_delta_chunk_scan_kernel<DP / 16>, dim3(hx, (a.V + 15) / 16, a.S), dim3(256), 0, st, a, rec);
  hipLaunchKernelGGL(gated_delta_chunk_finish_kernel, dim3(chunks, a.H), dim3(256), 0, st, a, DP, rec);
}

template <int KG, int NC, int DQ, int TC>
void launch_scan(const GatedDeltaArgs& a, const float4* vec, const float* vals, float* oraw, hipStream_t st) {
  constexpr int W = 4 * (64 / KG) * NC;
  hipLaunchKernelGGL((gated_delta_scan_kernel<KG, NC, DQ, TC>), dim3(a.S, a.H, (a.V + W - 1) / W), dim3(256), 0, st, a, vec, vals, oraw);
}

}  // namespace

size_t gated_delta_scratch_floats(int T, int S, int H, int D, int V) {
  const size_t tokens = (size_t)T * H * (4 * (size_t)D + 2 * (size_t)V);
  const size_t chunks = takes_chunks(T, S, D, V) ? (size_t)(T / CN + S) * H * chunk_floats(chunk_channels(D), V) : 0;
  return tokens > chunks ? tokens : chunks;
}

void launch_gated_delta(const GatedDeltaArgs& a, int T, float* scratch, hipStream_t st) {
  if (a.S <= 0 || a.H <= 0 || T <= 0) return;
  if (a.wide < 0 && a.taps <= CHUNK_MAX_TAPS && takes_chunks(T, a.S, a.D, a.V)) {
    const int DP = chunk_channels(a.D);
    if (DP == 32) launch_chunks<32>(a, T, scratch, st);
    else if (DP == 64) launch_chunks<64>(a, T, scratch, st);
    else launch_chunks<128>(a, T, scratch, st);
    return;
  }
  float4* vec = reinterpret_cast<float4*>(scratch);
  float* vals = scratch + 4 * (int64_t)T * a.H * a.D;
  float* oraw = vals + (int64_t)T * a.H * a.V;
  hipLaunchKernelGGL(gated_delta_prep_kernel, dim3(T, a.G), dim3(256), 2 * a.D * sizeof(float), st, a, vec, vals);
  // many (sequence, head, 32 columns) waves: the form with least work; few: the one with the shortest chain per token
  const bool wide = a.wide >= 0 ? a.wide > 0 : (int64_t)a.S * a.H * ((a.V + 31) / 32) >= 512;
  if (wide) {
    if (a.D <= 32) launch_scan<8, 4, 4, 8>(a, vec, vals, oraw, st);
    else if (a.D <= 64) launch_scan<8, 4, 8, 8>(a, vec, vals, oraw, st);
    else if (a.D <= 128) launch_scan<8, 4, 16, 4>(a, vec, vals, oraw, st);
    else launch_scan<8, 4, 32, 2>(a, vec, vals, oraw, st);
  } else {
    if (a.D <= 32) launch_scan<32, 1, 1, 8>(a, vec, vals, oraw, st);
    else if (a.D <= 64) launch_scan<32, 1, 2, 8>(a, vec, vals, oraw, st);
    else if (a.D <= 128) launch_scan<32, 1, 4, 8>(a, vec, vals, oraw, st);
    else launch_scan<32, 1, 8, 4>(a, vec, vals, oraw, st);
  }
  hipLaunchKernelGGL(gated_delta_finish_kernel, dim3(T, (a.H + 3) / 4), dim3(256), 0, st, a, oraw);
}

}  // namespace vgate
