// Kernels of a gated delta rule and around a Mamba-2 scan (gfx950): the delta
// rule's recurrence with a decay per key channel; the gates, the chunk-parallel
// matrix-core scan and the gated, grouped read-out norm of a state-space-duality
// mixer (whose token-serial scan, for single tokens, short portions and fp32
// models, is the scalar-gate mode of the diagonal-decay kernel in seqmix.hip).
//
// Numerics as in seqmix.hip: activations arrive in the model dtype T (bf16
// or fp32); unit norms, decays, step sizes, gates and state are fp32 in
// registers/LDS and rounded to T once, on store. bf16 models take the hardware
// exp/log, fp32 models the accurate functions.

#include "common.h"

// ------------------------------------------------------- gated delta rule ----
// Per sequence and head, state S [D, DV] fp32 in a per-sequence slot:
//   g_t = exp(-rate_h * softplus(z_t + z_bias)) per key channel, or one number
//         for all of them (HEAD_DECAY: z [T, H], z_bias [H]),
//   S <- diag(g_t) S;  u = sigmoid(beta_t) (v_t - S^T k_t);  S <- S + k_t u^T;
//   o_t = S^T q_t,
// with k_t and q_t unit vectors (x / sqrt(sum x^2 + 1e-6), q times q_scale).
//
// The read-out of the updated state is S_decayed^T q + (k.q) u, so both
// products with the state (with k for the correction, with q for the output)
// come from ONE walk over the decayed state and are reduced together; k.q is a
// number per token, computed when the token is staged. A token costs an element
// of S one multiply and three multiply-adds.
//
// Value columns are independent given k, q, g, so the grid splits DV: a
// workgroup owns 16 * NC columns of one (sequence, head). A column belongs to
// the 16 lanes of one DPP row, each with DPL key channels of NC adjacent
// columns in registers; the reduction over key channels is four DPP adds and
// never leaves the wave, so between the stages' barriers the four waves walk
// their columns freely. 16 tokens are staged in LDS at a time (the next stage's
// raw operands are fetched into registers before the token loop): a row of 16
// threads stages one token, which makes the unit norms and k.q row reductions
// too. Granules of GW channels are interleaved over the 16 lanes, so a wave's
// LDS reads of a token are contiguous (and broadcast over the four columns).
// Sequential over tokens: where a portion starts cannot change a sum's order.
constexpr int kDeltaTB = 16;

template <int CTRL>
DEVINL float dpp_add(float x) {
  return x + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), CTRL, 0xf, 0xf, true));
}

// sum over the 16 lanes of a DPP row, in every lane: quad permutes (xor 1,
// xor 2), then mirrors of half rows and rows, whose sources hold equal sums
DEVINL float row16_sum(float x) {
  x = dpp_add<0xB1>(x);
  x = dpp_add<0x4E>(x);
  x = dpp_add<0x141>(x);
  return dpp_add<0x140>(x);
}

template <bool FAST>
DEVINL float softplus_f(float x) {
  const float t = FAST ? __logf(1.0f + __expf(-fabsf(x))) : log1pf(expf(-fabsf(x)));
  return fmaxf(x, 0.f) + t;
}

template <typename T, int DPL, int NC, bool HEAD_DECAY>
__global__ __launch_bounds__(256) void gated_delta_kernel(
    float* __restrict__ o,                                  // [T, H, DV]
    const T* __restrict__ q, long q_stride, const T* __restrict__ k, long k_stride,
    const T* __restrict__ v, long v_stride, const T* __restrict__ z, long z_stride,
    const float* __restrict__ z_bias,                       // [H * D] or [H]
    const float* __restrict__ rate,                         // [H]
    const T* __restrict__ beta, long b_stride,              // [T, H]
    float* __restrict__ state,                              // [slots, H, D, DV]
    const int* __restrict__ cu, const int* __restrict__ slots, const int* __restrict__ fresh,
    int H, int hpk, int D, int DV, float q_scale) {
  constexpr bool FAST = sizeof(T) == 2;
  constexpr int DP = 16 * DPL;                 // padded key channels
  constexpr int GW = DPL < 4 ? DPL : 4;        // channels per granule
  constexpr int NG = DPL / GW;                 // granules per lane
  constexpr int COLS = 16 * NC;                // value columns per workgroup
  __shared__ __align__(16) float qs[kDeltaTB * DP];
  __shared__ __align__(16) float ks[kDeltaTB * DP];
  __shared__ __align__(16) float gs[HEAD_DECAY ? kDeltaTB : kDeltaTB * DP];
  __shared__ __align__(16) float vs[kDeltaTB * COLS];
  __shared__ float bs[kDeltaTB], kq[kDeltaTB];
  const int b = blockIdx.z, h = blockIdx.y, hk = h / hpk;
  const int row0 = cu[b], n = cu[b + 1] - row0;
  if (n <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int l = lane & 15;
  const int lc = (w * 4 + (lane >> 4)) * NC;   // first column within the workgroup
  const int c0 = blockIdx.x * COLS + lc;
  const long sbase = ((long)slots[b] * H + h) * D * (long)DV;
  const bool use_old = fresh[b] == 0;
  const bool vec_cols = NC == 4 && DV % 4 == 0;
  auto chan = [&](int i) { return ((i / GW) * 16 + l) * GW + i % GW; };
  float S[NC][DPL];
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int d = chan(i);
    const float* sp = state + sbase + (long)d * DV + c0;
    if constexpr (NC == 4) {
      if (vec_cols) {
        float4 s4 = make_float4(0.f, 0.f, 0.f, 0.f);
        if (use_old && d < D && c0 < DV) s4 = *reinterpret_cast<const float4*>(sp);
        S[0][i] = s4.x; S[1][i] = s4.y; S[2][i] = s4.z; S[3][i] = s4.w;
        continue;
      }
    }
#pragma unroll
    for (int c = 0; c < NC; ++c) S[c][i] = (use_old && d < D && c0 + c < DV) ? sp[c] : 0.f;
  }
  // staging: thread = (token tid / 16, lane l of its row): the row's granules
  // of q, k and z, NC of the v columns
  const int st = tid >> 4;
  constexpr int NZ = HEAD_DECAY ? 1 : DPL;     // decay logits per lane and token
  float zb[NZ];
#pragma unroll
  for (int i = 0; i < NZ; ++i)
    zb[i] = HEAD_DECAY ? z_bias[h] : chan(i) < D ? z_bias[h * D + chan(i)] : 0.f;
  const float rt = rate[h];
  float rq[DPL], rk[DPL], rz[NZ], rv[NC], rb = 0.f;
  auto fetch = [&](int t0) {
    const bool live = t0 + st < n;
    const long row = row0 + t0 + st;
#pragma unroll
    for (int i = 0; i < DPL; ++i) {
      const int d = chan(i);
      rq[i] = rk[i] = 0.f;
      if constexpr (!HEAD_DECAY) rz[i] = 0.f;
      if (live && d < D) {
        rq[i] = to_f32(q[row * q_stride + (long)hk * D + d]);
        rk[i] = to_f32(k[row * k_stride + (long)hk * D + d]);
        if constexpr (!HEAD_DECAY) rz[i] = to_f32(z[row * z_stride + (long)h * D + d]);
      }
    }
    if constexpr (HEAD_DECAY) rz[0] = live ? to_f32(z[row * z_stride + h]) : 0.f;
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int gc = blockIdx.x * COLS + l * NC + c;
      rv[c] = (live && gc < DV) ? to_f32(v[row * v_stride + (long)h * DV + gc]) : 0.f;
    }
    rb = live ? to_f32(beta[row * b_stride + h]) : 0.f;
  };
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += kDeltaTB) {
    const int nt = min(kDeltaTB, n - t0);
    __syncthreads();
    {
      float sq = 0.f, sk = 0.f, sqk = 0.f;
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        sq += rq[i] * rq[i];
        sk += rk[i] * rk[i];
        sqk += rq[i] * rk[i];
      }
      sq = row16_sum(sq);
      sk = row16_sum(sk);
      sqk = row16_sum(sqk);
      const float iq = q_scale / sqrtf(sq + 1e-6f), ik = 1.0f / sqrtf(sk + 1e-6f);
#pragma unroll
      for (int i = 0; i < DPL; ++i) {
        const int at = st * DP + chan(i);
        qs[at] = rq[i] * iq;
        ks[at] = rk[i] * ik;
        if constexpr (!HEAD_DECAY) {
          const float sp = softplus_f<FAST>(rz[i] + zb[i]);
          gs[at] = FAST ? __expf(-rt * sp) : expf(-rt * sp);
        }
      }
#pragma unroll
      for (int c = 0; c < NC; ++c) vs[st * COLS + l * NC + c] = rv[c];
      if (l == 0) {
        bs[st] = 1.0f / (1.0f + (FAST ? __expf(-rb) : expf(-rb)));
        kq[st] = sqk * iq * ik;
        if constexpr (HEAD_DECAY) {
          const float sp = softplus_f<FAST>(rz[0] + zb[0]);
          gs[st] = FAST ? __expf(-rt * sp) : expf(-rt * sp);
        }
      }
    }
    __syncthreads();
    if (t0 + kDeltaTB < n) fetch(t0 + kDeltaTB);
    for (int tt = 0; tt < nt; ++tt) {
      float kk[DPL], pk[NC], pq[NC];
#pragma unroll
      for (int c = 0; c < NC; ++c) pk[c] = pq[c] = 0.f;
      float gh = 1.f;
      if constexpr (HEAD_DECAY) gh = gs[tt];
#pragma unroll
      for (int g = 0; g < NG; ++g) {
        const int at = tt * DP + (g * 16 + l) * GW;
        float ga[GW], qa[GW];
        if constexpr (GW == 4) {
          const float4 g4 = HEAD_DECAY ? make_float4(gh, gh, gh, gh)
                                       : *reinterpret_cast<const float4*>(gs + at);
          const float4 k4 = *reinterpret_cast<const float4*>(ks + at);
          const float4 q4 = *reinterpret_cast<const float4*>(qs + at);
          ga[0] = g4.x; ga[1] = g4.y; ga[2] = g4.z; ga[3] = g4.w;
          qa[0] = q4.x; qa[1] = q4.y; qa[2] = q4.z; qa[3] = q4.w;
          kk[g * 4] = k4.x; kk[g * 4 + 1] = k4.y; kk[g * 4 + 2] = k4.z; kk[g * 4 + 3] = k4.w;
        } else {
#pragma unroll
          for (int e = 0; e < GW; ++e) {
            ga[e] = HEAD_DECAY ? gh : gs[at + e];
            kk[g * GW + e] = ks[at + e];
            qa[e] = qs[at + e];
          }
        }
#pragma unroll
        for (int e = 0; e < GW; ++e) {
          const int i = g * GW + e;
#pragma unroll
          for (int c = 0; c < NC; ++c) {
            if constexpr (!HEAD_DECAY) S[c][i] *= ga[e];
            pk[c] += S[c][i] * kk[i];
            pq[c] += S[c][i] * qa[e];
          }
        }
      }
      const float bt = bs[tt], kqt = kq[tt];
      float u[NC];
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        // one decay per head: it comes out of both products, and the state takes
        // it together with the write
        u[c] = bt * (vs[tt * COLS + lc + c] - gh * row16_sum(pk[c]));
        pq[c] = gh * row16_sum(pq[c]) + kqt * u[c];
      }
#pragma unroll
      for (int i = 0; i < DPL; ++i)
#pragma unroll
        for (int c = 0; c < NC; ++c)
          S[c][i] = (HEAD_DECAY ? gh * S[c][i] : S[c][i]) + kk[i] * u[c];
      if (l == 0) {
        float* op = o + ((long)(row0 + t0 + tt) * H + h) * DV + c0;
        if (vec_cols) {
          if constexpr (NC == 4)
            if (c0 < DV) *reinterpret_cast<float4*>(op) = make_float4(pq[0], pq[1], pq[2], pq[3]);
        } else {
#pragma unroll
          for (int c = 0; c < NC; ++c)
            if (c0 + c < DV) op[c] = pq[c];
        }
      }
    }
  }
#pragma unroll
  for (int i = 0; i < DPL; ++i) {
    const int d = chan(i);
    if (d >= D) continue;
    float* sp = state + sbase + (long)d * DV + c0;
    if constexpr (NC == 4) {
      if (vec_cols) {
        if (c0 < DV)
          *reinterpret_cast<float4*>(sp) = make_float4(S[0][i], S[1][i], S[2][i], S[3][i]);
        continue;
      }
    }
#pragma unroll
    for (int c = 0; c < NC; ++c)
      if (c0 + c < DV) sp[c] = S[c][i];
  }
}

// ---------------------------------------------------------- Mamba-2: gates ----
// step = softplus(dt + dt_bias) per (token, head); out [2, T, H] = the memory's
// decay exp(-rate * step) and its write strength step.
template <typename T>
__global__ void ssd_gates_kernel(float* __restrict__ out, const T* __restrict__ dt, long dt_stride,
                                 const float* __restrict__ dt_bias, const float* __restrict__ rate,
                                 long rows, int H) {
  constexpr bool FAST = sizeof(T) == 2;
  const long total = rows * H;
  for (long i = blockIdx.x * (long)blockDim.x + threadIdx.x; i < total;
       i += (long)gridDim.x * blockDim.x) {
    const long t = i / H;
    const int h = (int)(i % H);
    const float step = softplus_f<FAST>(to_f32(dt[t * dt_stride + h]) + dt_bias[h]);
    out[i] = FAST ? __expf(-rate[h] * step) : expf(-rate[h] * step);
    out[total + i] = step;
  }
}

// ------------------------------------- Mamba-2: chunk-parallel scan (bf16) ----
// S_t = e^(a_t) S_(t-1) + step_t B_t x_t^T, o_t = S_t^T C_t with a_t = -rate step_t
// has ONE decay per token, so over a chunk of 64 tokens with prefix sums
// cum_i = a_0 + .. + a_i (all <= 0, every difference below is <= 0 too):
//   o_i  = e^cum_i C_i S_prev + sum_(j <= i) (C_i . B_j) e^(cum_i - cum_j) step_j x_j
//   S    = e^cum_last S_prev  + sum_j B_j (e^(cum_last - cum_j) step_j x_j)^T
// four matrix products on v_mfma_f32_16x16x32_bf16 with fp32 accumulation.
// B, C and x are bf16 already; every fp32 factor (the state, the weighted
// scores, the weighted x) enters as TWO bf16 planes (value = hi + lo, lo the
// rounding remainder), the state itself stays in fp32 accumulators for the
// whole portion.
//
// Workgroup = 64 value columns of one (sequence, head), 8 waves. Wave (rt, hf):
// output rows 16 rt .. + 15 x columns 32 hf .. + 31 (and the scores of those
// rows with tokens 32 hf .. + 31), state rows NP/2 hf .. x columns 16 rt .. + 15.
// The next chunk's rows are fetched into registers during the products. LDS
// buffers whose lifetimes do not meet share their space (B rows / score planes;
// state planes / weighted-x planes). Rows past the portion's end carry step 0,
// which leaves state and prefix sums unchanged.
constexpr int kSsdQ = 64;
constexpr int kSsdKP = kSsdQ + 8;            // padded token stride of transposed tiles
typedef __attribute__((ext_vector_type(4))) short ssd_bf16x4;

DEVINL void split_bf16(float v, short& hi, short& lo) {
  const __hip_bfloat16 h = __float2bfloat16(v);
  hi = __bfloat16_as_short(h);
  lo = __bfloat16_as_short(__float2bfloat16(v - __bfloat162float(h)));
}

constexpr size_t ssd_chunk_lds(int nk) {
  const size_t ns = nk * 32 + 8;
  const size_t u1 = kSsdQ * ns > 8u * 16 * kSsdKP ? kSsdQ * ns : 8u * 16 * kSsdKP;
  const size_t u2 = 2 * 64 * ns > 2u * 64 * kSsdKP ? 2 * 64 * ns : 2u * 64 * kSsdKP;
  return 2 * (u1 + u2 + (size_t)nk * 32 * kSsdKP + 64 * kSsdKP) + 2 * kSsdQ * 4;
}

template <int NK>                            // states padded to NK * 32
__global__ __launch_bounds__(512, 4) void ssd_chunk_scan_kernel(
    float* __restrict__ o,                                   // [T, H, DV]
    const __hip_bfloat16* __restrict__ Cm, long c_stride, const __hip_bfloat16* __restrict__ Bm,
    long b_stride, const __hip_bfloat16* __restrict__ x, long x_stride,
    const float* __restrict__ steps,                         // [T, H]
    const float* __restrict__ rate,                          // [H]
    float* __restrict__ state,                               // [slots, H, N, DV]
    const int* __restrict__ cu, const int* __restrict__ slots, const int* __restrict__ fresh,
    int H, int hpg, int N, int DV) {
  extern __shared__ __align__(16) unsigned char ssd_smem[];
  constexpr int NP = NK * 32, NS = NP + 8, KP = kSsdKP, Q = kSsdQ;
  constexpr int NG = NK > 1 ? NK / 2 : 1;                    // B granules per thread
  constexpr int U1 = Q * NS > 8 * 16 * KP ? Q * NS : 8 * 16 * KP;
  constexpr int U2 = 2 * 64 * NS > 2 * 64 * KP ? 2 * 64 * NS : 2 * 64 * KP;
  short* Bs = reinterpret_cast<short*>(ssd_smem);            // [Q][NS]
  short* Ps = Bs;                                            // [4 row tiles][hi, lo][16][KP]
  short* St = Bs + U1;                                       // [hi, lo][64][NS]
  short* Xw = St;                                            // [hi, lo][64][KP]
  short* Bt = St + U2;                                       // [NP][KP]
  short* Xt = Bt + NP * KP;                                  // [64][KP]
  float* cum = reinterpret_cast<float*>(Xt + 64 * KP);       // [Q]
  float* stp = cum + Q;                                      // [Q]
  const int b = blockIdx.z, h = blockIdx.y, c0 = blockIdx.x * 64;
  const int row0 = cu[b], n = cu[b + 1] - row0;
  if (n <= 0) return;
  const int g = h / hpg;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int rt = w & 3, hf = w >> 2, col = lane & 15, kgrp = lane >> 4;
  const float rt_h = -rate[h];
  const long sbase = ((long)slots[b] * H + h) * N * (long)DV;
  const bool use_old = fresh[b] == 0;
  const int vcol = c0 + rt * 16 + col;                       // this lane's state column
  sm_f32x4 S[NK];
#pragma unroll
  for (int r = 0; r < NK; ++r)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int nn = (hf * NK + r) * 16 + kgrp * 4 + e;
      S[r][e] = (use_old && nn < N && vcol < DV) ? state[sbase + (long)nn * DV + vcol] : 0.f;
    }
  // staged token and granule: a wave holds one granule of all 64 tokens, so its
  // transposing LDS stores are 64 adjacent elements
  const int sj = lane, sub = w;
  const sm_bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  sm_bf16x8 rc[NK], rb[NG], rx = zero8;      // rc: this lane's C operands, straight from memory
  float rstep = 0.f;
  auto fetch = [&](int t0) {
    const bool live = t0 + sj < n;
    const long row = row0 + t0 + sj;
#pragma unroll
    for (int i = 0; i < NG; ++i) {
      const int d8 = (sub + 8 * i) * 8;
      rb[i] = zero8;
      if (live && d8 < N)
        rb[i] = *reinterpret_cast<const sm_bf16x8*>(Bm + row * b_stride + (long)g * N + d8);
    }
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) {
      const int t = t0 + rt * 16 + col, d8 = ks * 32 + kgrp * 8;
      rc[ks] = t < n && d8 < N
          ? *reinterpret_cast<const sm_bf16x8*>(Cm + (row0 + t) * c_stride + (long)g * N + d8) : zero8;
    }
    rx = zero8;
    if (live && c0 + sub * 8 < DV)
      rx = *reinterpret_cast<const sm_bf16x8*>(x + row * x_stride + (long)h * DV + c0 + sub * 8);
    rstep = t0 + lane < n ? steps[(long)(row0 + t0 + lane) * H + h] : 0.f;
  };
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += Q) {
    __syncthreads();                         // the previous chunk's tiles are read
#pragma unroll
    for (int i = 0; i < NG; ++i) {
      const int d8 = (sub + 8 * i) * 8;
      if (d8 < NP) {
        *reinterpret_cast<sm_bf16x8*>(Bs + sj * NS + d8) = rb[i];
#pragma unroll
        for (int e = 0; e < 8; ++e) Bt[(d8 + e) * KP + sj] = rb[i][e];
      }
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) Xt[(sub * 8 + e) * KP + sj] = rx[e];
#pragma unroll
    for (int r = 0; r < NK; ++r) {
      ssd_bf16x4 hi, lo;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        short a, c;
        split_bf16(S[r][e], a, c);
        hi[e] = a;
        lo[e] = c;
      }
      const int at = (rt * 16 + col) * NS + (hf * NK + r) * 16 + kgrp * 4;
      *reinterpret_cast<ssd_bf16x4*>(St + at) = hi;
      *reinterpret_cast<ssd_bf16x4*>(St + 64 * NS + at) = lo;
    }
    float cl = rt_h * rstep;                 // inclusive prefix sum over the wave's 64 lanes
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const float up = __shfl_up(cl, off, WAVE);
      if (lane >= off) cl += up;
    }
    if (w == 0) {
      cum[lane] = cl;
      stp[lane] = rstep;
    }
    const float cum_last = __shfl(cl, 63, WAVE);
    const sm_bf16x8 xg = rx;                 // this chunk's x granule, weighted below
    sm_bf16x8 cf[NK];
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) cf[ks] = rc[ks];
    __syncthreads();
    if (t0 + Q < n) fetch(t0 + Q);
    sm_f32x4 s[2], y[2];
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) s[ct] = y[ct] = sm_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) {
#pragma unroll
      for (int ct = 0; ct < 2; ++ct) {
        const int at = ((hf * 2 + ct) * 16 + col) * NS + ks * 32 + kgrp * 8;
        const sm_bf16x8 bf = *reinterpret_cast<const sm_bf16x8*>(Bs + at);
        const sm_bf16x8 sh = *reinterpret_cast<const sm_bf16x8*>(St + at);
        const sm_bf16x8 sl = *reinterpret_cast<const sm_bf16x8*>(St + 64 * NS + at);
        s[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cf[ks], bf, s[ct], 0, 0, 0);
        y[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cf[ks], sh, y[ct], 0, 0, 0);
        y[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cf[ks], sl, y[ct], 0, 0, 0);
      }
    }
    float ci[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) ci[e] = cum[rt * 16 + kgrp * 4 + e];
    __syncthreads();                         // B rows and state planes are read
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) {
      const int j = (hf * 2 + ct) * 16 + col;
      const float cj = cum[j], pj = stp[j];
      short* pr = Ps + rt * 2 * 16 * KP + j;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = kgrp * 4 + e;
        const float p = j <= rt * 16 + i ? s[ct][e] * __expf(ci[e] - cj) * pj : 0.f;
        split_bf16(p, pr[i * KP], pr[(16 + i) * KP]);
        y[ct][e] *= __expf(ci[e]);
      }
    }
    {
      const float wj = __expf(cum_last - cum[sj]) * stp[sj];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int at = (sub * 8 + e) * KP + sj;
        split_bf16(__uint_as_float((unsigned)(unsigned short)xg[e] << 16) * wj, Xw[at],
                   Xw[64 * KP + at]);
      }
    }
    __syncthreads();
    const float dl = __expf(cum_last);
#pragma unroll
    for (int r = 0; r < NK; ++r) S[r] *= dl;
#pragma unroll
    for (int k2 = 0; k2 < Q / 32; ++k2) {
      const int ko = k2 * 32 + kgrp * 8;
      const short* pr = Ps + (rt * 2 * 16 + col) * KP + ko;
      const sm_bf16x8 ph = *reinterpret_cast<const sm_bf16x8*>(pr);
      const sm_bf16x8 pl = *reinterpret_cast<const sm_bf16x8*>(pr + 16 * KP);
#pragma unroll
      for (int ct = 0; ct < 2; ++ct) {
        const sm_bf16x8 xf = *reinterpret_cast<const sm_bf16x8*>(Xt + ((hf * 2 + ct) * 16 + col) * KP + ko);
        y[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph, xf, y[ct], 0, 0, 0);
        y[ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, xf, y[ct], 0, 0, 0);
      }
      const short* xr = Xw + (rt * 16 + col) * KP + ko;
      const sm_bf16x8 wh = *reinterpret_cast<const sm_bf16x8*>(xr);
      const sm_bf16x8 wl = *reinterpret_cast<const sm_bf16x8*>(xr + 64 * KP);
#pragma unroll
      for (int r = 0; r < NK; ++r) {
        const sm_bf16x8 bf = *reinterpret_cast<const sm_bf16x8*>(Bt + ((hf * NK + r) * 16 + col) * KP + ko);
        S[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf, wh, S[r], 0, 0, 0);
        S[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf, wl, S[r], 0, 0, 0);
      }
    }
#pragma unroll
    for (int ct = 0; ct < 2; ++ct) {
      const int c = c0 + (hf * 2 + ct) * 16 + col;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int t = t0 + rt * 16 + kgrp * 4 + e;
        if (t < n && c < DV) o[((long)(row0 + t) * H + h) * DV + c] = y[ct][e];
      }
    }
  }
#pragma unroll
  for (int r = 0; r < NK; ++r)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int nn = (hf * NK + r) * 16 + kgrp * 4 + e;
      if (nn < N && vcol < DV) state[sbase + (long)nn * DV + vcol] = S[r][e];
    }
}

// ------------------------------------------------------- Mamba-2: read-out ----
// y = (o + D_h x) * silu(z), then RMS norm in `groups` equal parts of `width`
// channels, times weight. A part belongs to a team of TEAM threads (64: a wave,
// four parts per workgroup; 256: a workgroup), V adjacent channels of one head
// per thread and step; up to kSsdKeep steps' results stay in registers between
// the sum and the store, what lies beyond is computed again.
constexpr int kSsdKeep = 4;

template <typename T, int V>
DEVINL void ssd_out_values(const float* __restrict__ o, const T* __restrict__ x,
                           const T* __restrict__ z, float d, float* y) {
  float ov[V], xv[V], zv[V];
  if constexpr (V == 4 && sizeof(T) == 2) {
    const float4 o4 = *reinterpret_cast<const float4*>(o);
    const Vec4<T> x4 = load8(x), z4 = load8(z);
    ov[0] = o4.x; ov[1] = o4.y; ov[2] = o4.z; ov[3] = o4.w;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      xv[e] = to_f32(x4.data[e]);
      zv[e] = to_f32(z4.data[e]);
    }
  } else {
#pragma unroll
    for (int e = 0; e < V; ++e) {
      ov[e] = o[e];
      xv[e] = to_f32(x[e]);
      zv[e] = to_f32(z[e]);
    }
  }
#pragma unroll
  for (int e = 0; e < V; ++e) {
    const float sg = 1.0f / (1.0f + (sizeof(T) == 2 ? __expf(-zv[e]) : expf(-zv[e])));
    y[e] = (ov[e] + d * xv[e]) * zv[e] * sg;
  }
}

template <typename T, int TEAM, int V>
__global__ __launch_bounds__(256) void ssd_out_gate_norm_kernel(
    T* __restrict__ out, const float* __restrict__ o, const T* __restrict__ x, long x_stride,
    const float* __restrict__ Dp, const T* __restrict__ z, long z_stride,
    const T* __restrict__ weight, int width, int groups, long rows, int DV, float eps) {
  __shared__ float red[4];
  const int member = TEAM == 64 ? (threadIdx.x & 63) : threadIdx.x;
  const long row = TEAM == 64 ? blockIdx.x * 4L + (threadIdx.x >> 6) : blockIdx.x;
  if (TEAM == 64 && row >= rows) return;
  const long tok = row / groups;
  const int first = (int)(row % groups) * width;       // the part's first channel
  const float* op = o + tok * groups * (long)width + first;
  const T* xp = x + tok * x_stride + first;
  const T* zp = z + tok * z_stride + first;
  T* outp = out + tok * groups * (long)width + first;
  float keep[kSsdKeep][V];
  float ss = 0.f;
#pragma unroll
  for (int s = 0; s < kSsdKeep; ++s) {
    const int i = (s * TEAM + member) * V;
    if (i < width) {
      ssd_out_values<T, V>(op + i, xp + i, zp + i, Dp[(first + i) / DV], keep[s]);
#pragma unroll
      for (int e = 0; e < V; ++e) ss += keep[s][e] * keep[s][e];
    }
  }
  for (int i = (kSsdKeep * TEAM + member) * V; i < width; i += TEAM * V) {
    float y[V];
    ssd_out_values<T, V>(op + i, xp + i, zp + i, Dp[(first + i) / DV], y);
#pragma unroll
    for (int e = 0; e < V; ++e) ss += y[e] * y[e];
  }
  ss = TEAM == 64 ? wave_reduce_sum(ss) : block_reduce_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / width + eps);
  auto put = [&](int i, const float* y) {
    if constexpr (V == 4 && sizeof(T) == 2) {
      const Vec4<T> w4 = load8(weight + first + i);
      Vec4<T> r;
#pragma unroll
      for (int e = 0; e < V; ++e) r.data[e] = from_f32<T>(y[e] * inv * to_f32(w4.data[e]));
      *reinterpret_cast<int2*>(outp + i) = *reinterpret_cast<const int2*>(r.data);
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e)
        outp[i + e] = from_f32<T>(y[e] * inv * to_f32(weight[first + i + e]));
    }
  };
#pragma unroll
  for (int s = 0; s < kSsdKeep; ++s) {
    const int i = (s * TEAM + member) * V;
    if (i < width) put(i, keep[s]);
  }
  for (int i = (kSsdKeep * TEAM + member) * V; i < width; i += TEAM * V) {
    float y[V];
    ssd_out_values<T, V>(op + i, xp + i, zp + i, Dp[(first + i) / DV], y);
    put(i, y);
  }
}
