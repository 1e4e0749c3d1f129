// Selective scan: a diagonal recurrence per (channel, state) with an input-dependent step, fp32 states [channel][state]
// in a state slot between steps:
//   d = softplus(dt);  S[c, n] <- exp(d_c A[c, n]) S[c, n] + d_c x_c B_n;  y_c = sum_n S[c, n] C_n + D_c x_c
//   out_c = y_c silu(z_c)
// x is what a short causal convolution (short_conv.h) and silu made of the projection, B and C are rows of the step's
// projection of x. A comes as A log2(e), so a decay is one exp2.
//   short_conv   one thread per (token, eight channels): convolution, bias, silu (scalar form for other alignments).
//   scan         lane = (channel, one of LPC parts of its states), NS states in registers; per token and state one exp2,
//                two FMAs and a product, LPC lanes meet in log2(LPC) lane exchanges. Tokens are staged through LDS TC at
//                a time (softplus, D x and the gate taken there) while the next TC load into registers; outputs leave through
//                LDS, so that the stores run over whole rows of channels. One barrier per TC tokens.
// Long steps run the scan over chunks of CH tokens in parallel:
//   local   every chunk from a zero state: its local state L_c and its sum of steps s_c
//   carry   per sequence, chunk after chunk: I_0 = slot state, I_(c+1) = exp(s_c A) I_c + L_c (the same recurrence taken
//           CH tokens at a time, all fp32); the slot receives the last one
//   output  every chunk again from its true initial state, now with outputs
// The launch that writes the slot's state also rewrites the kept convolution inputs. A portion that starts at position 0
// starts from zero, so a reused slot needs no clearing.
#include "common.h"
#include "seq_launchers.h"
#include "short_conv.h"

namespace vgate {
namespace {

__device__ __forceinline__ float silu_f(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
template <int CTRL>
__device__ __forceinline__ float dpp(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, false));
}
// sum over aligned groups of LPC (4 or 16) lanes
template <int LPC>
__device__ __forceinline__ float part_sum(float v) {
  if (LPC == 4) {
    v += dpp<0xB1>(v);   // quad_perm [1, 0, 3, 2]
    v += dpp<0x4E>(v);   // quad_perm [2, 3, 0, 1]
  } else {
    v += dpp<0x128>(v); v += dpp<0x124>(v); v += dpp<0x122>(v); v += dpp<0x121>(v);  // row_ror 8, 4, 2, 1
  }
  return v;
}

// VEC channels per thread (8: 16-B pieces, host-checked alignment; 1: any)
template <int VEC>
__global__ __launch_bounds__(256) void short_conv_kernel(ShortConvArgs p) {
  const int t = blockIdx.x;
  if (t >= p.query_start[p.S]) return;
  const int s = seq_of_row(p.query_start, p.S, t);
  const int slot = p.state_slots[s];
  if (slot < 0) return;
  const int t0 = p.query_start[s], pos0 = p.context_lens[s] - (p.query_start[s + 1] - t0);
  const float* kept = p.kept + (int64_t)slot * (p.taps - 1) * p.C;
  for (int c = (blockIdx.y * 256 + threadIdx.x) * VEC; c < p.C; c += gridDim.y * 256 * VEC) {
    if (VEC == 1) {
      float y = short_conv_at(p.x, p.ldx, p.f32, c, p.w, p.C, c, p.b != nullptr ? p.b[c] : 0.f, kept, p.C, c, t, t0, pos0, p.taps);
      if (p.act) y = silu_f(y);
      const int64_t oi = (int64_t)t * p.ldo + c;
      if (p.f32) reinterpret_cast<float*>(p.out)[oi] = y;
      else reinterpret_cast<bf16_t*>(p.out)[oi] = f2bf(y);
    } else {
      float y[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) y[e] = p.b != nullptr ? p.b[c + e] : 0.f;
      for (int i = 0; i < p.taps; ++i) {
        const int tt = t - (p.taps - 1) + i;
        float v[8];
        if (tt >= t0) {
          unpack8(ld16(reinterpret_cast<const bf16_t*>(p.x) + (int64_t)tt * p.ldx + c), v);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] = pos0 > 0 ? kept[(int64_t)(tt - t0 + p.taps - 1) * p.C + c + e] : 0.f;
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) y[e] = fmaf(p.w[(int64_t)i * p.C + c + e], v[e], y[e]);
      }
      if (p.act)
#pragma unroll
        for (int e = 0; e < 8; ++e) y[e] = silu_f(y[e]);
      *reinterpret_cast<uint4*>(reinterpret_cast<bf16_t*>(p.out) + (int64_t)t * p.ldo + c) = pack8(y);
    }
  }
}

enum { SCAN_WHOLE = 0, SCAN_LOCAL = 1, SCAN_OUTPUT = 2 };

__device__ __forceinline__ bool locate_chunk(const SelectiveScanArgs& p, int CH, int bx, int& s, int& t0, int& t1) {
  int base = 0;
  for (int i = 0; i < p.S; ++i) {
    const int a = p.query_start[i], b = p.query_start[i + 1];
    const int nc = (p.state_slots[i] < 0 || b <= a) ? 0 : (b - a + CH - 1) / CH;
    if (bx < base + nc) {
      s = i; t0 = a + (bx - base) * CH; t1 = min(b, t0 + CH);
      return true;
    }
    base += nc;
  }
  return false;
}

// MODE WHOLE: blockIdx.x a sequence, its whole portion from its slot. LOCAL / OUTPUT: blockIdx.x one chunk of CH tokens
// (chunks of all sequences numbered in order). blockIdx.y: 256 / LPC channels.
template <int LPC, int NS, int MODE, bool F32>
__global__ __launch_bounds__(256) void selective_scan_kernel(SelectiveScanArgs p, int CH, float* __restrict__ cstate,
                                                              float* __restrict__ cstep) {
  constexpr int TC = 8, CPB = 256 / LPC, NT = LPC * NS;
  constexpr int NX = (TC * CPB + 255) / 256, NB = (TC * NT + 255) / 256;
  constexpr bool OUT = MODE != SCAN_LOCAL;
  __shared__ __attribute__((aligned(16))) float lb[2][TC][NT], lc[OUT ? 2 : 1][TC][NT];
  __shared__ __attribute__((aligned(16))) float4 lt[2][TC][CPB];   // {d, d x, D x, silu(z)} of a token and channel
  __shared__ float ly[OUT ? 2 : 1][TC][CPB];
  int s = blockIdx.x, t0, t1;
  if (MODE == SCAN_WHOLE) {
    t0 = p.query_start[s]; t1 = p.query_start[s + 1];
    if (p.state_slots[s] < 0 || t1 <= t0) return;
  } else if (!locate_chunk(p, CH, blockIdx.x, s, t0, t1)) {
    return;
  }
  const int tid = threadIdx.x, cl = tid / LPC, part = tid % LPC;
  const int cb = blockIdx.y * CPB, c = cb + cl;
  const int C = p.C, N = p.N, n0 = part * NS;
  const int slot = p.state_slots[s];
  const bool from_zero = MODE == SCAN_LOCAL || (MODE == SCAN_WHOLE && p.context_lens[s] - (t1 - t0) <= 0);
  float* sp = (MODE == SCAN_WHOLE ? p.state + (int64_t)slot * C * N : cstate + (int64_t)blockIdx.x * C * N) + (int64_t)c * N + n0;
  const float* ap = p.A + (int64_t)c * N + n0;
  float S[NS], A[NS], steps = 0.f;
#pragma unroll
  for (int j = 0; j < NS; ++j) {
    const bool on = c < C && n0 + j < N;
    A[j] = on ? ap[j] : 0.f;
    S[j] = (on && !from_zero) ? sp[j] : 0.f;
  }
  float Dc[NX], pd[NX], px[NX], pz[NX], pb[NB], pc[NB];
#pragma unroll
  for (int r = 0; r < NX; ++r) {
    const int cc = cb + (tid + 256 * r) % CPB;
    Dc[r] = (OUT && cc < C) ? p.D[cc] : 0.f;
  }
  // rows past the portion's end and channels past the last are read from clamped places (their results are never used);
  // states past the last have B = C = 0
  constexpr int RX = 256 / CPB;   // tokens apart of a thread's pieces
  const int xcol = min(cb + tid % CPB, C - 1);
  const int row = tid / CPB;
  auto fetch = [&](int tb) {
#pragma unroll
    for (int r = 0; r < NX; ++r) {
      const int t = min(tb + row + RX * r, t1 - 1);
      pd[r] = p.dt[(int64_t)t * p.lddt + xcol];
      px[r] = conv_ldx(p.x, (int64_t)t * p.ldx + xcol, F32 ? 1 : 0);
      if (OUT) pz[r] = conv_ldx(p.z, (int64_t)t * p.ldz + xcol, F32 ? 1 : 0);
    }
#pragma unroll
    for (int r = 0; r < NB; ++r) {
      const int e = tid + 256 * r, n = e % NT;
      const int64_t o = (int64_t)min(tb + e / NT, t1 - 1) * p.ldbc + min(n, N - 1);
      pb[r] = conv_ldx(p.B, o, F32 ? 1 : 0);
      if (OUT) pc[r] = conv_ldx(p.Cm, o, F32 ? 1 : 0);
      if (n >= N) pb[r] = pc[r] = 0.f;
    }
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int r = 0; r < NX; ++r) {
      const int e = tid + 256 * r;
      if (e < TC * CPB) {
        const float d = softplus_f(pd[r]);
        (&lt[buf][0][0])[e] = make_float4(d, d * px[r], OUT ? Dc[r] * px[r] : 0.f, OUT ? silu_f(pz[r]) : 0.f);
      }
    }
#pragma unroll
    for (int r = 0; r < NB; ++r) {
      const int e = tid + 256 * r;
      if (e < TC * NT) {
        (&lb[buf][0][0])[e] = pb[r];
        if (OUT) (&lc[OUT ? buf : 0][0][0])[e] = pc[r];
      }
    }
  };
  auto store = [&](int tb, int nt, int buf) {  // a finished tile's rows of channels
    for (int e = tid; e < nt * CPB; e += 256) {
      const int cc = cb + e % CPB;
      if (cc >= C) continue;
      const float o = (&ly[OUT ? buf : 0][0][0])[e];
      const int64_t oi = (int64_t)(tb + e / CPB) * p.ldo + cc;
      if (F32) reinterpret_cast<float*>(p.out)[oi] = o;
      else reinterpret_cast<bf16_t*>(p.out)[oi] = f2bf(o);
    }
  };
  fetch(t0);
  put(0);
  lds_barrier();
  int buf = 0;
  for (int tb = t0; tb < t1; tb += TC) {
    const bool more = tb + TC < t1;
    if (more) fetch(tb + TC);
    if (OUT && tb > t0) store(tb - TC, TC, buf ^ 1);
    const int nt = min(TC, t1 - tb);
#pragma unroll
    for (int i = 0; i < TC; ++i) {
      if (i >= nt) break;
      const float4 x = lt[buf][i][cl];
      float y = 0.f;
#pragma unroll
      for (int j = 0; j < NS; ++j) {
        S[j] = fmaf(__builtin_amdgcn_exp2f(x.x * A[j]), S[j], x.y * lb[buf][i][n0 + j]);
        if (OUT) y = fmaf(S[j], lc[OUT ? buf : 0][i][n0 + j], y);
      }
      if (OUT) {
        y = part_sum<LPC>(y);
        if (part == 0) ly[OUT ? buf : 0][i][cl] = (y + x.z) * x.w;
      } else {
        steps += x.x;
      }
    }
    if (more) put(buf ^ 1);  // (every wave left that buffer before the last barrier)
    lds_barrier();
    if (!more && OUT) store(tb, nt, buf);
    buf ^= 1;
  }
  if (MODE == SCAN_OUTPUT) return;
#pragma unroll
  for (int j = 0; j < NS; ++j)
    if (c < C && n0 + j < N) sp[j] = S[j];
  if (MODE == SCAN_LOCAL) {
    if (part == 0 && c < C) cstep[(int64_t)blockIdx.x * C + c] = steps;
  } else if (part == 0 && c < C) {
    short_conv_keep(p.xin, p.ldxin, p.f32, c, p.kept + (int64_t)slot * (p.taps - 1) * C, C, c, t0, t1,
                    p.context_lens[s] - (t1 - t0), p.taps);
  }
}

// one thread per (sequence, channel, state): cstate[chunk] becomes the state the chunk starts from, the slot the state
// after the last one; threads of state 0 rewrite the kept convolution inputs
__global__ __launch_bounds__(256) void selective_carry_kernel(SelectiveScanArgs p, int CH, float* __restrict__ cstate,
                                                               const float* __restrict__ cstep) {
  const int s = blockIdx.x;
  const int slot = p.state_slots[s];
  const int t0 = p.query_start[s], t1 = p.query_start[s + 1];
  if (slot < 0 || t1 <= t0) return;
  int base = 0;
  for (int i = 0; i < s; ++i) {
    const int a = p.query_start[i], b = p.query_start[i + 1];
    base += (p.state_slots[i] < 0 || b <= a) ? 0 : (b - a + CH - 1) / CH;
  }
  const int nc = (t1 - t0 + CH - 1) / CH, C = p.C, N = p.N;
  const int pos0 = p.context_lens[s] - (t1 - t0);
  const int64_t CN = (int64_t)C * N;
  float* sp = p.state + (int64_t)slot * CN;
  for (int64_t e = (int64_t)blockIdx.y * 256 + threadIdx.x; e < CN; e += (int64_t)gridDim.y * 256) {
    const int c = (int)(e / N);
    const float A = p.A[e];
    float cur = pos0 <= 0 ? 0.f : sp[e];
    for (int k = 0; k < nc; ++k) {
      float* cs = cstate + (base + k) * CN + e;
      const float loc = *cs;
      *cs = cur;
      cur = fmaf(__builtin_amdgcn_exp2f(cstep[(int64_t)(base + k) * C + c] * A), cur, loc);
    }
    sp[e] = cur;
    if (e % N == 0)
      short_conv_keep(p.xin, p.ldxin, p.f32, c, p.kept + (int64_t)slot * (p.taps - 1) * C, C, c, t0, t1, pos0, p.taps);
  }
}

template <int LPC, int NS, bool F32>
void launch_scan_as(const SelectiveScanArgs& a, int T, float* cstate, float* cstep, hipStream_t st) {
  constexpr int CPB = 256 / LPC;
  const int CH = selective_scan_chunk_size(T, a.S), cols = (a.C + CPB - 1) / CPB;
  if (CH <= 0) {
    hipLaunchKernelGGL((selective_scan_kernel<LPC, NS, SCAN_WHOLE, F32>), dim3(a.S, cols), dim3(256), 0, st, a, 0, nullptr, nullptr);
    return;
  }
  const int chunks = T / CH + a.S;
  hipLaunchKernelGGL((selective_scan_kernel<LPC, NS, SCAN_LOCAL, F32>), dim3(chunks, cols), dim3(256), 0, st, a, CH, cstate, cstep);
  const int64_t ey = ((int64_t)a.C * a.N + 255) / 256;
  hipLaunchKernelGGL(selective_carry_kernel, dim3(a.S, (unsigned)(ey < 1024 ? ey : 1024)), dim3(256), 0, st, a, CH, cstate, cstep);
  hipLaunchKernelGGL((selective_scan_kernel<LPC, NS, SCAN_OUTPUT, F32>), dim3(chunks, cols), dim3(256), 0, st, a, CH, cstate, cstep);
}
template <int LPC, int NS>
void launch_scan(const SelectiveScanArgs& a, int T, float* cstate, float* cstep, hipStream_t st) {
  if (a.f32) launch_scan_as<LPC, NS, true>(a, T, cstate, cstep, st);
  else launch_scan_as<LPC, NS, false>(a, T, cstate, cstep, st);
}

}  // namespace

void launch_short_conv(const ShortConvArgs& a, hipStream_t st) {
  if (a.T <= 0 || a.S <= 0 || a.C <= 0) return;
  const bool vec = !a.f32 && a.C % 8 == 0 && a.ldx % 8 == 0 && a.ldo % 8 == 0 && (reinterpret_cast<uintptr_t>(a.x) & 15) == 0 &&
                   (reinterpret_cast<uintptr_t>(a.out) & 15) == 0;
  const int per = vec ? 256 * 8 : 256;
  int gy = (a.C + per - 1) / per;
  if (gy > 64) gy = 64;
  if (vec) hipLaunchKernelGGL(short_conv_kernel<8>, dim3(a.T, gy), dim3(256), 0, st, a);
  else hipLaunchKernelGGL(short_conv_kernel<1>, dim3(a.T, gy), dim3(256), 0, st, a);
}

int selective_scan_chunk_size(int T, int S) {
  // steps of a few tokens per sequence (decoding, short portions): one pass per sequence; long ones: chunks
  return T >= 256 && T >= 64 * S ? 64 : 0;
}
size_t selective_scan_scratch_floats(int T, int S, int C, int N) {
  const int CH = selective_scan_chunk_size(T, S);
  return CH > 0 ? (size_t)(T / CH + S) * C * ((size_t)N + 1) : 0;
}

void launch_selective_scan(const SelectiveScanArgs& a, int T, float* scratch, hipStream_t st) {
  if (a.S <= 0 || a.C <= 0 || T <= 0) return;
  const int CH = selective_scan_chunk_size(T, a.S);
  float* cstate = scratch;
  float* cstep = CH > 0 ? scratch + (size_t)(T / CH + a.S) * a.C * a.N : nullptr;
  if (a.N <= 16) launch_scan<4, 4>(a, T, cstate, cstep, st);
  else if (a.N <= 32) launch_scan<4, 8>(a, T, cstate, cstep, st);
  else if (a.N <= 64) launch_scan<4, 16>(a, T, cstate, cstep, st);
  else if (a.N <= 128) launch_scan<16, 8>(a, T, cstate, cstep, st);
  else launch_scan<16, 16>(a, T, cstate, cstep, st);
}

}  // namespace vgate
