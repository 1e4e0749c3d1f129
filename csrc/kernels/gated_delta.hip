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
//   finish token parallel: head RMS norm, norm weight, output gate, store; the block of a portion's last token also
//          rewrites the slot's kept convolution inputs.
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

// one workgroup per token; waves take heads in turn
__global__ __launch_bounds__(256) void gated_delta_finish_kernel(GatedDeltaArgs p, const float* __restrict__ oraw) {
  const int t = blockIdx.x;
  if (t >= p.query_start[p.S]) return;
  const int H = p.H, V = p.V, D = p.D, GD = p.G * D, HV = H * V;
  const int s = seq_of_row(p.query_start, p.S, t);
  const int slot = p.state_slots[s];
  if (slot < 0) return;
  const int wv = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const float* o = oraw + (int64_t)t * HV;
  for (int h = wv; h < H; h += 4) {
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
  for (int e = threadIdx.x; e < NC; e += 256) {
    const void* x = e < GD ? p.q : (e < 2 * GD ? p.k : p.v);
    const int64_t ld = e < GD ? p.ldq : (e < 2 * GD ? p.ldk : p.ldv);
    short_conv_keep(x, ld, p.f32, e < GD ? e : (e < 2 * GD ? e - GD : e - 2 * GD), kept, NC, e, t0, t1, pos0, p.taps);
  }
}

template <int KG, int NC, int DQ, int TC>
void launch_scan(const GatedDeltaArgs& a, const float4* vec, const float* vals, float* oraw, hipStream_t st) {
  constexpr int W = 4 * (64 / KG) * NC;
  hipLaunchKernelGGL((gated_delta_scan_kernel<KG, NC, DQ, TC>), dim3(a.S, a.H, (a.V + W - 1) / W), dim3(256), 0, st, a, vec, vals, oraw);
}

}  // namespace

size_t gated_delta_scratch_floats(int T, int H, int D, int V) { return (size_t)T * H * (4 * (size_t)D + 2 * (size_t)V); }

void launch_gated_delta(const GatedDeltaArgs& a, int T, float* scratch, hipStream_t st) {
  if (a.S <= 0 || a.H <= 0 || T <= 0) return;
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
  hipLaunchKernelGGL(gated_delta_finish_kernel, dim3(T), dim3(256), 0, st, a, oraw);
}

}  // namespace vgate
