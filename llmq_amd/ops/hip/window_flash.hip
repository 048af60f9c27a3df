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

// ------------------------------------------------------------ single tokens --
// The same attention for one new token per sequence: the query heads that share
// a kv head (16 at a time) are the columns of S^T = K Q^T and O^T = V^T P^T on
// v_mfma_f32_16x16x32_bf16 (A: row = lane%16, k = 8*(lane/16)..+7; B: column =
// lane%16; C: column = lane%16, rows 4*(lane/16)+r), so every key row is read
// once for all of them. Slot order of a 32-key step: slot 8 h + 4 b + i = key
// 16 b + 4 h + i.
//
// Waves are independent: each takes every (4 * n_split)-th tile of 16 NK keys, K
// operands straight from memory, V through a wave-private transposed LDS tile,
// the next tile's rows in flight during the current tile's products. The four
// waves' partials merge through LDS; with n_split > 1 a workgroup writes its
// unnormalised output, maximum (natural log domain) and sum to `part`
// [sequence, head, split, DV + 2] for attn_merge_splits_kernel.
constexpr size_t window_decode_lds(int dt, int nk) {
  const size_t tiles = 4 * sizeof(short) * (size_t)dt * 16 * (nk * 16 + 8);
  const size_t merge = 4 * sizeof(float) * (size_t)16 * (dt * 16 + 2);
  return tiles > merge ? tiles : merge;
}

// KS: key channels padded to 32 KS; DT: value channels padded to 16 DT.
template <int KS, int DT, int NK>
__global__ __launch_bounds__(256, (KS <= 4 ? 2 : 1)) void window_decode_kernel(
    __hip_bfloat16* __restrict__ out, long out_stride,
    const __hip_bfloat16* __restrict__ q, long q_stride,
    const __hip_bfloat16* __restrict__ gate, long g_stride, int gate_cols,
    const __hip_bfloat16* __restrict__ k_cache, const __hip_bfloat16* __restrict__ v_cache,
    int v_row, const int* __restrict__ block_tables, int bt_stride,
    const int* __restrict__ context_lens, int H, int G, int D, int DV, int bs_shift, int window,
    float scale_log2, const float* __restrict__ sink, int n_split, float* __restrict__ part) {
  extern __shared__ __align__(16) unsigned char wd_smem[];
  constexpr int KT = 16 * NK, KP = KT + 8;
  constexpr int KG = KT / 4, GW = 64 / KG;               // key groups and granules of a V task
  constexpr int NV = (DT * 2 + GW - 1) / GW;             // V tasks per lane
  const int hp = H / G, ng = (hp + 15) / 16;
  const int sp = blockIdx.x % n_split, grp = blockIdx.x / n_split;
  const int g = grp / ng, c0 = (grp % ng) * 16;          // kv head, its first query head here
  const int heads = min(16, hp - c0), h0 = g * hp + c0;
  const int b = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int col = lane & 15, grp4 = lane >> 4;
  short* Vt = reinterpret_cast<short*>(wd_smem) + w * (DT * 16 * KP);    // [16 DT][KP]
  const int pos = context_lens[b] - 1;
  const int lo = max(0, pos - window + 1);
  const int* bt = block_tables + (long)b * bt_stride;
  const int bs_mask = (1 << bs_shift) - 1;
  const wf_bf16x8 zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  wf_bf16x8 qf[KS];
  {
    const __hip_bfloat16* qr = q + (long)b * q_stride + (long)(h0 + col) * D;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d8 = ks * 32 + grp4 * 8;
      qf[ks] = col < heads && d8 < D ? *reinterpret_cast<const wf_bf16x8*>(qr + d8) : zero8;
    }
  }
  const int sg = lane % GW, kg = lane / GW;
  const int kpos = (kg >> 3) * 32 + (kg & 3) * 8 + ((kg >> 2) & 1) * 4;
  auto row_of = [&](int key) -> long {
    return (((long)bt[key >> bs_shift] * G + g) << bs_shift) + (key & bs_mask);
  };
  wf_bf16x8 kf[NK][KS], vf[NV][4];
  auto fetch = [&](int kt) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int key = kt + i * 16 + col;
      const bool live = key <= pos;
      const __hip_bfloat16* kr = k_cache + (live ? row_of(key) : 0L) * D;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const int d8 = ks * 32 + grp4 * 8;
        kf[i][ks] = live && d8 < D ? *reinterpret_cast<const wf_bf16x8*>(kr + d8) : zero8;
      }
    }
    const int key = kt + kg * 4;
    const __hip_bfloat16* vr = v_cache + (key <= pos ? row_of(key) : 0L) * v_row;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d8 = (i * GW + sg) * 8;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        vf[i][e] = d8 < DV && key + e <= pos
            ? *reinterpret_cast<const wf_bf16x8*>(vr + (long)e * v_row + d8) : zero8;
    }
  };
  float m = -INFINITY, l = 0.f;              // log2 domain
  sm_f32x4 o[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) o[dt] = sm_f32x4{0.f, 0.f, 0.f, 0.f};
  const int step = KT * 4 * n_split;
  int kt = (lo / KT) * KT + (sp * 4 + w) * KT;
  if (kt <= pos) fetch(kt);
  for (; kt <= pos; kt += step) {
    sm_f32x4 s[NK];
#pragma unroll
    for (int i = 0; i < NK; ++i) s[i] = sm_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ++ks)
#pragma unroll
      for (int i = 0; i < NK; ++i)
        s[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i][ks], qf[ks], s[i], 0, 0, 0);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d8 = (i * GW + sg) * 8;
      if (d8 < DV) {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          wf_u32x2 v4;
          v4[0] = (unsigned)(unsigned short)vf[i][0][j] | ((unsigned)(unsigned short)vf[i][1][j] << 16);
          v4[1] = (unsigned)(unsigned short)vf[i][2][j] | ((unsigned)(unsigned short)vf[i][3][j] << 16);
          *reinterpret_cast<wf_u32x2*>(Vt + (d8 + j) * KP + kpos) = v4;
        }
      }
    }
    if (kt + step <= pos) fetch(kt + step);
    if (kt < lo || kt + KT - 1 > pos) {
#pragma unroll
      for (int i = 0; i < NK; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = kt + i * 16 + grp4 * 4 + r;
          s[i][r] = key >= lo && key <= pos ? s[i][r] : -INFINITY;
        }
    }
    float tmax = s[0][0];
#pragma unroll
    for (int i = 0; i < NK; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) tmax = fmaxf(tmax, s[i][r]);
    tmax = fmaxf(tmax, __shfl_xor(tmax, 16, WAVE));
    tmax = fmaxf(tmax, __shfl_xor(tmax, 32, WAVE));
    const float m_new = fmaxf(m, tmax * scale_log2);         // scale > 0
    const float mb = m_new > -INFINITY ? m_new : 0.f;
    const float alpha = __builtin_amdgcn_exp2f(m - mb);      // m = -inf -> 0
    l *= alpha;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) o[dt] *= alpha;
    m = m_new;
    // the tile's writes come before its reads: one wave, LDS in order
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int j = 0; j < NK / 2; ++j) {       // 32 keys per step
      wf_u32x4 hi, lw;
#pragma unroll
      for (int e = 0; e < 8; e += 2) {
        const float p0 = __builtin_amdgcn_exp2f(fmaf(s[2 * j + e / 4][e % 4], scale_log2, -mb));
        const float p1 = __builtin_amdgcn_exp2f(fmaf(s[2 * j + e / 4][e % 4 + 1], scale_log2, -mb));
        l += p0 + p1;
        const unsigned b0 = __float_as_uint(p0), b1 = __float_as_uint(p1);
        hi[e / 2] = __builtin_amdgcn_perm(b1, b0, 0x07060302u);
        const wf_f32x2 rest = {p0 - __uint_as_float(b0 & 0xffff0000u),
                               p1 - __uint_as_float(b1 & 0xffff0000u)};
        lw[e / 2] = __builtin_bit_cast(unsigned, __builtin_convertvector(rest, wf_bfx2));
      }
      const wf_bf16x8 ph = __builtin_bit_cast(wf_bf16x8, hi), pl = __builtin_bit_cast(wf_bf16x8, lw);
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const wf_bf16x8 va = *reinterpret_cast<const wf_bf16x8*>(
            Vt + (dt * 16 + col) * KP + j * 32 + grp4 * 8);
        o[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, ph, o[dt], 0, 0, 0);
        o[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, pl, o[dt], 0, 0, 0);
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  // merge of the four waves: [wave][column][DV, m, l] fp32 over the V tiles
  __syncthreads();
  float* Mg = reinterpret_cast<float*>(wd_smem);
  constexpr int MW = DT * 16 + 2;
  float* mine = Mg + (w * 16 + col) * MW;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int r = 0; r < 4; ++r) mine[dt * 16 + grp4 * 4 + r] = o[dt][r];
  if (grp4 == 0) {
    mine[DT * 16] = m;
    mine[DT * 16 + 1] = l;
  }
  __syncthreads();
  for (int idx = tid; idx < heads * DV; idx += 256) {
    const int hh = idx / DV, c = idx % DV, h = h0 + hh;
    const float* pw = Mg + hh * MW;
    float top = -INFINITY;
#pragma unroll
    for (int ww = 0; ww < 4; ++ww) top = fmaxf(top, pw[ww * 16 * MW + DT * 16]);
    const float sk = sink && n_split == 1 ? sink[h] * 1.44269504088896340736f : -INFINITY;
    top = fmaxf(top, sk);
    const float tb = top > -INFINITY ? top : 0.f;
    float a = 0.f, ll = __builtin_amdgcn_exp2f(sk - tb);
#pragma unroll
    for (int ww = 0; ww < 4; ++ww) {
      const float f = __builtin_amdgcn_exp2f(pw[ww * 16 * MW + DT * 16] - tb);
      a += pw[ww * 16 * MW + c] * f;
      ll += pw[ww * 16 * MW + DT * 16 + 1] * f;
    }
    if (n_split > 1) {
      float* pr = part + (((long)b * H + h) * n_split + sp) * (DV + 2);
      pr[c] = a;
      if (c == 0) {
        pr[DV] = top * 0.69314718055994530942f;
        pr[DV + 1] = ll;
      }
    } else {
      out[(long)b * out_stride + (long)h * DV + c] = __float2bfloat16(
          a / ll * head_gate(gate, (long)b * g_stride, gate_cols, h, c));
    }
  }
}

// Merge of key splits: out[b, h] = sum_s o_s e^(m_s - M) / sum_s l_s e^(m_s - M),
// M = max_s m_s, a sink joining as one more l; a split that saw no key has
// m = -inf and counts nothing. One wave per (sequence, head), lanes over value
// channels.
__global__ __launch_bounds__(256) void attn_merge_splits_kernel(
    __hip_bfloat16* __restrict__ out, long out_stride, const float* __restrict__ part,
    long pairs, int H, int DV, int n_split, const float* __restrict__ sink,
    const __hip_bfloat16* __restrict__ gate, long g_stride, int gate_cols) {
  const long pair = blockIdx.x * 4L + (threadIdx.x >> 6);
  if (pair >= pairs) return;
  const int lane = threadIdx.x & 63;
  const long b = pair / H;
  const int h = (int)(pair % H);
  const float* pp = part + pair * n_split * (long)(DV + 2);
  // a lane reads one split's maximum and sum (at most 64 splits)
  const float ms = lane < n_split ? pp[lane * (DV + 2) + DV] : -INFINITY;
  const float ls = lane < n_split ? pp[lane * (DV + 2) + DV + 1] : 0.f;
  float M = wave_reduce_max(ms);
  if (sink) M = fmaxf(M, sink[h]);
  const float f = ms > -INFINITY ? expf(ms - M) : 0.f;
  const float L = wave_reduce_sum(ls * f) + (sink ? expf(sink[h] - M) : 0.f);
  const float inv = 1.0f / L;
  for (int c = lane; c - lane < DV; c += 64) {      // all lanes stay for the shuffles
    float a = 0.f;
    for (int s = 0; s < n_split; ++s) {
      const float fs = __shfl(f, s, WAVE);
      if (c < DV) a += pp[s * (DV + 2) + c] * fs;
    }
    if (c < DV)
      out[b * out_stride + (long)h * DV + c] =
          __float2bfloat16(a * inv * head_gate(gate, b * g_stride, gate_cols, h, c));
  }
}
