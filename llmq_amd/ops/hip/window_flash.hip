// Softmax attention of bf16 prompt portions over the paged cache on the matrix
// cores (gfx950): causal or sliding window, optional softmax sink and output
// gate, values of their own or the first channels of the key rows. The plain
// case of the attention of seqmix.hip, which keeps every other option (learned
// biases, score caps, kept first tokens, sigmoid weights, decode rows).
//
// Workgroup = 128 query rows x 1 head, 4 waves x 32 rows, key tiles of 64.
// Both products run TRANSPOSED on v_mfma_f32_32x32x16_bf16, S^T = K Q^T and
// O^T = V^T P^T (A: row = lane%32, k = 8*(lane/32)..+7; B: column = lane%32;
// C: column = lane%32, rows 8*(r/4) + 4*(lane/32) + r%4), so a lane owns ONE
// query: its scores, running maximum, sum and rescale factor stay in the lane
// (one exchange with the other half of the wave per tile), and the weights are
// already where the second product wants them - they never pass through LDS.
// For that the keys of the contraction come in the order in which S^T leaves
// them: 16 keys per step, slot 8 h + 4 b + i of a step = key 8 b + 4 h + i, and
// V^T sits in LDS in that order, one 16-byte read per operand.
//
// The weights enter as TWO bf16 planes (p = hi + lo), hi cut off, lo the
// rounded remainder: 16 mantissa bits. Scores, mask and softmax are fp32 in the
// log2 domain; tiles that every row of a wave sees whole skip the mask.
//
// Staging: a lane takes 4 consecutive keys x 8 channels (16 bytes each); K goes
// to LDS row-major, V transposed by packing 4 keys of a channel into 8 bytes.
// The next tile is fetched into registers before the current tile's products.
//
// Grid: heaviest (latest) query tiles first, and consecutive workgroups - which
// the dispatcher deals out to the XCDs in turn - take (sequence, head) pairs
// far apart, so each XCD keeps the keys of few sequences in its own L2 and all
// XCDs get query tiles of the same weight.

#include "common.h"

constexpr int kWfQT = 128;
constexpr int kWfKT = 64;
constexpr int kWfKP = kWfKT + 8;             // padded key stride of the V^T tile
typedef __attribute__((ext_vector_type(8))) short wf_bf16x8;
typedef __attribute__((ext_vector_type(2))) unsigned wf_u32x2;
typedef __attribute__((ext_vector_type(4))) unsigned wf_u32x4;
typedef __attribute__((ext_vector_type(16))) float wf_f32x16;
typedef __attribute__((ext_vector_type(2))) float wf_f32x2;
typedef __attribute__((ext_vector_type(2))) __bf16 wf_bfx2;

constexpr size_t window_flash_lds(int ks, int dt) {
  return sizeof(short) * ((size_t)kWfKT * (ks * 16 + 8) + (size_t)dt * 32 * kWfKP);
}

// KS: key channels padded to 16 KS (even); DT: value channels padded to 32 DT.
template <int KS, int DT, bool ALIAS>
__global__ __launch_bounds__(256, (KS <= 8 ? 2 : 1)) void window_flash_kernel(
    __hip_bfloat16* __restrict__ out, long out_stride,
    const __hip_bfloat16* __restrict__ q, long q_stride,
    const __hip_bfloat16* __restrict__ gate, long g_stride, int gate_cols,
    const __hip_bfloat16* __restrict__ k_cache, const __hip_bfloat16* __restrict__ v_cache,
    const int* __restrict__ block_tables, int bt_stride,
    const int* __restrict__ cu_q, const int* __restrict__ q_start,
    int B, int H, int G, int D, int DV, int bs_shift, int window, float scale_log2,
    const float* __restrict__ sink, int n_qt) {
  extern __shared__ __align__(16) unsigned char wf_smem[];
  constexpr int DS = KS * 16 + 8;
  constexpr int KW = KS / 2;                 // wave tasks (4 granules x 64 keys) of K
  constexpr int WT = KW + (ALIAS ? 0 : DT);  // and of V, if it is not in K's rows
  constexpr int NT = (WT + 3) / 4;
  short* Ks = reinterpret_cast<short*>(wf_smem);       // [KT][DS]
  short* Vt = Ks + kWfKT * DS;                         // [32 DT][KP]
  const int nb = H * B;
  const int n = blockIdx.x % nb;
  const int pair = nb % 8 == 0 ? (n % 8) * (nb / 8) + n / 8 : n;
  const int b = pair / H, h = pair % H;
  const int r0 = (n_qt - 1 - blockIdx.x / nb) * kWfQT;
  const int row0 = cu_q[b];
  const int nq = cu_q[b + 1] - row0;
  if (r0 >= nq) return;
  const int rows = min(kWfQT, nq - r0);
  const int pos0 = q_start[b] + r0;
  const int pos_last = pos0 + rows - 1;
  const int g = h / (H / G);
  const int tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 31, half = lane >> 5;
  const int* bt = block_tables + (long)b * bt_stride;
  const wf_bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};

  // this lane's query
  const int qrow = w * 32 + col;
  const int ipos = qrow < rows ? pos0 + qrow : -1;     // -1: sees nothing
  const int lpos = max(0, ipos - window + 1);
  wf_bf16x8 qf[KS];
  {
    const __hip_bfloat16* qr = q + (long)(row0 + r0 + qrow) * q_stride + (long)h * D;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d8 = ks * 16 + half * 8;
      qf[ks] = qrow < rows && d8 < D ? *reinterpret_cast<const wf_bf16x8*>(qr + d8) : zero8;
    }
  }
  const int wave_first = pos0 + w * 32;
  const int wave_last = min(pos_last, wave_first + 31);
  const int wave_lo = max(0, wave_first - window + 1);       // first key any row sees
  const int wave_all = max(0, wave_last - window + 1);       // first key every row sees

  // staging: lane = (granule lane%4, key group lane/4)
  const int sg = lane & 3, kg = lane >> 2;
  const int kpos = (kg >> 2) * 16 + (kg & 1) * 8 + ((kg >> 1) & 1) * 4;   // V^T place of its keys
  const int bs_mask = (1 << bs_shift) - 1;
  wf_bf16x8 st[NT][4];
  auto fetch = [&](int kt) {
    const int key = kt + kg * 4;
    long base = 0;
    if (key <= pos_last)
      base = (((long)bt[key >> bs_shift] * G + g) << bs_shift) + (key & bs_mask);
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int wt = w + 4 * i;
      const bool is_v = wt >= KW;
      const int d8 = ((is_v ? wt - KW : wt) * 4 + sg) * 8;
      const int width = is_v ? DV : D;
      const __hip_bfloat16* src = (is_v ? v_cache : k_cache) + base * width + d8;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        st[i][e] = wt < WT && d8 < width && key + e <= pos_last
            ? *reinterpret_cast<const wf_bf16x8*>(src + (long)e * width) : zero8;
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int wt = w + 4 * i;
      if (wt >= WT) continue;
      const bool is_v = wt >= KW;
      const int d8 = ((is_v ? wt - KW : wt) * 4 + sg) * 8;
      if (!is_v) {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          *reinterpret_cast<wf_bf16x8*>(Ks + (kg * 4 + e) * DS + d8) = st[i][e];
      }
      if (is_v || (ALIAS && d8 < DV)) {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          wf_u32x2 v4;
          v4[0] = (unsigned)(unsigned short)st[i][0][j] | ((unsigned)(unsigned short)st[i][1][j] << 16);
          v4[1] = (unsigned)(unsigned short)st[i][2][j] | ((unsigned)(unsigned short)st[i][3][j] << 16);
          *reinterpret_cast<wf_u32x2*>(Vt + (d8 + j) * kWfKP + kpos) = v4;
        }
      }
    }
  };

  float m = -INFINITY, l = 0.f;              // log2 domain
  wf_f32x16 o[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[dt][r] = 0.f;

  const int kt0 = max(0, pos0 - window + 1) & ~(kWfKT - 1);
  fetch(kt0);
  for (int kt = kt0; kt <= pos_last; kt += kWfKT) {
    __syncthreads();                         // the previous tile is read
    stage();
    __syncthreads();
    if (kt + kWfKT <= pos_last) fetch(kt + kWfKT);
    if (w * 32 >= rows || kt > wave_last || kt + kWfKT - 1 < wave_lo) continue;
    wf_f32x16 s[2];
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int r = 0; r < 16; ++r) s[t][r] = 0.f;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const wf_bf16x8 kf = *reinterpret_cast<const wf_bf16x8*>(
            Ks + (t * 32 + col) * DS + ks * 16 + half * 8);
        s[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[ks], s[t], 0, 0, 0);
      }
    }
    if (kt + kWfKT - 1 > wave_first || kt < wave_all) {
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = kt + t * 32 + (r >> 2) * 8 + half * 4 + (r & 3);
          s[t][r] = key <= ipos && key >= lpos ? s[t][r] : -INFINITY;
        }
    }
    float tmax = s[0][0];
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int r = 0; r < 16; ++r) tmax = fmaxf(tmax, s[t][r]);
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, WAVE));
    const float m_new = fmaxf(m, tmax * scale_log2);         // scale > 0
    const float mb = m_new > -INFINITY ? m_new : 0.f;
    if (__any(m_new > m)) {
      const float alpha = __builtin_amdgcn_exp2f(m - mb);    // m = -inf -> 0
      l *= alpha;
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) o[dt] *= alpha;
      m = m_new;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {            // 16 keys per step
      const int t = j >> 1, u = (j & 1) * 8;
      wf_u32x4 hi, lo;
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const float p0 = __builtin_amdgcn_exp2f(fmaf(s[t][u + e], scale_log2, -mb));
        const float p1 = __builtin_amdgcn_exp2f(fmaf(s[t][u + e + 1], scale_log2, -mb));
        l += p0 + p1;
        const unsigned b0 = __float_as_uint(p0), b1 = __float_as_uint(p1);
        hi[e / 2] = __builtin_amdgcn_perm(b1, b0, 0x07060302u);
        const wf_f32x2 rest = {p0 - __uint_as_float(b0 & 0xffff0000u),
                               p1 - __uint_as_float(b1 & 0xffff0000u)};
        lo[e / 2] = __builtin_bit_cast(unsigned, __builtin_convertvector(rest, wf_bfx2));
      }
      const wf_bf16x8 ph = __builtin_bit_cast(wf_bf16x8, hi), pl = __builtin_bit_cast(wf_bf16x8, lo);
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const wf_bf16x8 vf = *reinterpret_cast<const wf_bf16x8*>(
            Vt + (dt * 32 + col) * kWfKP + j * 16 + half * 8);
        o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, ph, o[dt], 0, 0, 0);
        o[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pl, o[dt], 0, 0, 0);
      }
    }
  }
  l += __shfl_xor(l, 32, WAVE);
  if (qrow >= rows) return;
  float f = 1.f;
  if (sink) {
    const float sk = sink[h] * 1.44269504088896340736f;
    const float top = fmaxf(m, sk);
    f = __builtin_amdgcn_exp2f(m - top);
    l = l * f + __builtin_amdgcn_exp2f(sk - top);
  }
  f /= l;
  const long trow = row0 + r0 + qrow;
  if (gate && gate_cols == 1) f /= 1.0f + __expf(-to_f32(gate[trow * g_stride + h]));
  const __hip_bfloat16* gr =
      gate && gate_cols != 1 ? gate + trow * g_stride + (long)h * DV : nullptr;
  __hip_bfloat16* orow = out + trow * out_stride + (long)h * DV;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int r = 0; r < 16; r += 4) {
      const int c = dt * 32 + (r >> 2) * 8 + half * 4;
      if (c >= DV) continue;
      Vec4<__hip_bfloat16> v;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float y = o[dt][r + e] * f;
        if (gr) y /= 1.0f + __expf(-to_f32(gr[c + e]));
        v.data[e] = __float2bfloat16(y);
      }
      *reinterpret_cast<int2*>(orow + c) = *reinterpret_cast<const int2*>(v.data);
    }
}
