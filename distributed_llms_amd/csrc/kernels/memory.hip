// Prompt chunks of the exponentially gated matrix memory on the matrix cores (ops/linattn.py memory_scan):
//
//     m_t = max(f_t + m_(t-1), i_t);  S <- e^(f_t + m_(t-1) - m_t) S + e^(i_t - m_t) k v^T;  n likewise with k alone
//     o = S^T q / (max(|n . q|, e^-m_t) + den_eps)
//
// in blocks of C = 64 tokens.  With F_t = f_1 + .. + f_t inside the block and S, n, m the state before it,
//
//     m_t  = max(F_t + m, max_(s <= t)(F_t - F_s + i_s)),   alpha_t = e^(F_t + m - m_t)
//     P_ts = (q_t . k_s) e^(F_t - F_s + i_s - m_t)  (s <= t, else 0)
//     S^T q = alpha_t S^T q_t + sum_s P_ts v_s,             n . q = alpha_t n . q_t + sum_s P_ts
//     S <- alpha_C S + sum_s w_s k_s v_s^T, n likewise,     w_s = e^(F_C - F_s + i_s - m_C)
//
// so one block costs four small matrix products instead of 64 dependent steps.  One workgroup (4 waves) per
// (sequence, head, slice of 64 CT value columns) walks the sequence's blocks; a wave owns 16 CT value columns.
//
//   * S lives in float32 MFMA accumulators (row = key channel, column = value column) for the whole walk.  The
//     accumulator layout hands a lane the channels 4g .. 4g + 3 of two 16-channel tiles; q and k are staged in LDS
//     with their channels in that order, so the accumulators ARE the B operand of q S: no exchange of state.
//   * Operands that are float32 (S in the read-out, w_s v_s in the update) are cut into three bf16 pieces of 8
//     significand bits each -- together the float32 value -- and P into two (16 bits, as the softmax weights of
//     attention_window.hip); q, k and v are bf16 as projected.  All sums are float32.
//   * K and V are needed with 8 consecutive TOKENS per lane (K^T, V^T): every thread transposes an 8 x 8 block in
//     registers (byte permutes) on its way to LDS.
//   * The next block's loads are in flight during the products; its gates (a max-plus scan over 64 lanes) are made
//     by wave 0, which has the least of the causal q k^T, during the current block.
#include <math.h>

#include "common.h"
#include "launchers.h"

namespace dllm {

constexpr int kMlC = 64;                 // tokens per block
typedef uint32_t ml_u32x4 __attribute__((ext_vector_type(4)));

// e = hi + mid + lo exactly: upper 16 bits of e, of the remainder, and the rest (bf16 by truncation each)
__device__ __forceinline__ void ml_split3(const float (&e)[8], bf16x8 (&p)[3]) {
  ml_u32x4 h, m, l;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    uint32_t a = __float_as_uint(e[2 * i]), b = __float_as_uint(e[2 * i + 1]);
    h[i] = __builtin_amdgcn_perm(b, a, 0x07060302u);
    const float ra = e[2 * i] - __uint_as_float(a & 0xffff0000u), rb = e[2 * i + 1] - __uint_as_float(b & 0xffff0000u);
    a = __float_as_uint(ra), b = __float_as_uint(rb);
    m[i] = __builtin_amdgcn_perm(b, a, 0x07060302u);
    const float sa = ra - __uint_as_float(a & 0xffff0000u), sb = rb - __uint_as_float(b & 0xffff0000u);
    l[i] = __builtin_amdgcn_perm(__float_as_uint(sb), __float_as_uint(sa), 0x07060302u);
  }
  p[0] = __builtin_bit_cast(bf16x8, h), p[1] = __builtin_bit_cast(bf16x8, m), p[2] = __builtin_bit_cast(bf16x8, l);
}

// Place of channel quad qd (4 channels) inside its 32-channel block: accumulator order (see above)
__device__ __forceinline__ int ml_quad(int qd) { return 8 * (qd & 3) + 4 * (qd >> 2); }

// NKB: 32-channel blocks of a key (D <= 32 NKB); CT: 16-column tiles per wave.
template <int NKB, int CT>
__global__ void __launch_bounds__(256, 2) ml_chunk_kernel(
    float* __restrict__ o, const bf16* __restrict__ proj, long ld, int qcol, int kcol, int vcol, int icol, int fcol,
    const float* __restrict__ i_bias, const float* __restrict__ f_bias, float cap, float q_scale, float den_eps,
    float* __restrict__ s_state, float* __restrict__ n_state, float* __restrict__ m_state, float* __restrict__ nm_ws,
    const int32_t* __restrict__ cu, const int32_t* __restrict__ positions, const int32_t* __restrict__ slots, int H, int D,
    int Dv) {
  constexpr int C = kMlC, DP = 32 * NKB, NR = 2 * NKB, COLS = 64 * CT;
  constexpr int QP = DP + 8, TP = C + 8;               // row pitches in elements (+ 16 bytes: rows on different banks)
  constexpr int KSZ = C * QP > 2 * C * TP ? C * QP : 2 * C * TP;
  constexpr int NBLK = DP + COLS, BPT = (NBLK + 255) / 256;      // 8 x 8 blocks: DP of K, COLS of V
  constexpr float kL2e = 1.4426950408889634f;
  __shared__ __attribute__((aligned(16))) bf16 sq[C * QP];       // Q rows, channels in accumulator order
  __shared__ __attribute__((aligned(16))) bf16 sk[KSZ];          // K rows likewise; then P hi | P lo [token][token]
  __shared__ __attribute__((aligned(16))) bf16 skt[DP * TP];     // K^T [channel][token]
  __shared__ __attribute__((aligned(16))) bf16 svt[COLS * TP];   // V^T [column][token]
  __shared__ __attribute__((aligned(16))) float g_af[2][C], g_gs[2][C], g_al[2][C], g_em[2][C], g_w[2][C];
  __shared__ __attribute__((aligned(16))) float rs[C], qn[C], sn[DP];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int lo = cu[b], hi = cu[b + 1];
  if (hi <= lo) return;
  const int wave = tid >> 6, lane = tid & 63, col = lane & 15, grp = lane >> 4;
  const int col0 = blockIdx.z * COLS, vbase = 16 * CT * wave;    // first column of the workgroup / wave (in the slice)
  const size_t srow = (size_t)slots[b] * H + h;
  const bool resume = positions[lo] > 0;
  const int d8 = D >> 3;
  // ---- state in
  f32x4 S[NR][CT];
#pragma unroll
  for (int ct = 0; ct < CT; ++ct) {
    const int v = col0 + vbase + 16 * ct + col;
    const float* row = s_state + (srow * Dv + (v < Dv ? v : 0)) * D;
#pragma unroll
    for (int rt = 0; rt < NR; ++rt) {
      const int d = 16 * rt + 4 * grp;
      S[rt][ct] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (resume && v < Dv && d < D) S[rt][ct] = *reinterpret_cast<const f32x4*>(row + d);
    }
  }
  for (int d = tid; d < DP; d += 256)
    sn[(d & ~31) + ml_quad((d & 31) >> 2) + (d & 3)] = resume && d < D ? n_state[srow * D + d] : 0.f;
  float m = resume ? m_state[srow] : 0.f;              // wave 0 carries it
  // padding channels of Q, K and K^T are written here once (K's are overwritten by P: finite, against Q's zeros)
  for (int i = tid; i < C * QP; i += 256) sq[i] = (bf16)0.f;
  for (int i = tid; i < KSZ; i += 256) sk[i] = (bf16)0.f;
  for (int i = tid; i < DP * TP; i += 256) skt[i] = (bf16)0.f;
  for (int i = tid; i < COLS * TP; i += 256) svt[i] = (bf16)0.f;
  // ---- loads of a block: Q pieces of 8 channels, 8 x 8 blocks of K and V (8 tokens x 8 channels)
  bf16x8 qreg[NKB], breg[BPT][8];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int r = 0; r < NKB; ++r) {
      const int idx = tid + 256 * r, t = idx / (DP / 8), c = idx - t * (DP / 8);
#pragma unroll
      for (int j = 0; j < 8; ++j) qreg[r][j] = (bf16)0.f;
      if (t0 + t < hi && c < d8) qreg[r] = *reinterpret_cast<const bf16x8*>(proj + (size_t)(t0 + t) * ld + qcol + h * D + 8 * c);
    }
#pragma unroll
    for (int r = 0; r < BPT; ++r) {
      const int blk = tid + 256 * r;
      const bool isk = blk < DP;
      const int w8 = isk ? DP / 8 : COLS / 8, bb = isk ? blk : blk - DP;
      const int tb = bb / w8, c = bb - tb * w8;
      const bool ok = blk < NBLK && (isk ? c < d8 : col0 + 8 * c < Dv);
      const long at = isk ? (long)kcol + h * D + 8 * c : (long)vcol + h * Dv + col0 + 8 * c;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
#pragma unroll
        for (int e = 0; e < 8; ++e) breg[r][j][e] = (bf16)0.f;
        if (ok && t0 + 8 * tb + j < hi) breg[r][j] = *reinterpret_cast<const bf16x8*>(proj + (size_t)(t0 + 8 * tb + j) * ld + at);
      }
    }
  };
  auto put_row = [&](bf16* dst, int t, int c, bf16x8 v) {        // 8 channels 8c .. of token t, accumulator order
    bf16* p = dst + t * QP + 32 * (c >> 2) + ml_quad(2 * (c & 3));
    *reinterpret_cast<bf16x4*>(p) = bf16x4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<bf16x4*>(p + 8) = bf16x4{v[4], v[5], v[6], v[7]};
  };
  auto stage = [&]() {
#pragma unroll
    for (int r = 0; r < NKB; ++r) {
      const int idx = tid + 256 * r, t = idx / (DP / 8), c = idx - t * (DP / 8);
      if (c < d8) put_row(sq, t, c, qreg[r]);
    }
#pragma unroll
    for (int r = 0; r < BPT; ++r) {
      const int blk = tid + 256 * r;
      if (blk >= NBLK) continue;
      const bool isk = blk < DP;
      const int w8 = isk ? DP / 8 : COLS / 8, bb = isk ? blk : blk - DP;
      const int tb = bb / w8, c = bb - tb * w8;
      if (isk) {
        if (c >= d8) continue;
#pragma unroll
        for (int j = 0; j < 8; ++j) put_row(sk, 8 * tb + j, c, breg[r][j]);
      }
      bf16* dst = (isk ? skt : svt) + (size_t)(8 * c) * TP + 8 * tb;
      ml_u32x4 w[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) w[j] = __builtin_bit_cast(ml_u32x4, breg[r][j]);
#pragma unroll
      for (int p = 0; p < 4; ++p) {
        ml_u32x4 e0, e1;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          e0[j] = __builtin_amdgcn_perm(w[2 * j + 1][p], w[2 * j][p], 0x05040100u);
          e1[j] = __builtin_amdgcn_perm(w[2 * j + 1][p], w[2 * j][p], 0x07060302u);
        }
        *reinterpret_cast<ml_u32x4*>(dst + (2 * p) * TP) = e0;
        *reinterpret_cast<ml_u32x4*>(dst + (2 * p + 1) * TP) = e1;
      }
    }
  };
  // ---- gates of a block (wave 0; a lane per token; lanes past the chunk's end pass the state on unchanged)
  const float bi = i_bias[h], bfg = f_bias[h];
  float zi = 0.f, zf = 0.f;
  auto fetch_gates = [&](int t0) {
    const bf16* row = proj + (size_t)min(t0 + lane, hi - 1) * ld;
    zi = bf2f(row[icol + h]), zf = bf2f(row[fcol + h]);
  };
  auto make_gates = [&](int t0, int buf) {
    const bool ok = t0 + lane < hi;
    const float z = cap * tanhf((zf + bfg) / cap);
    const float ig = ok ? cap * tanhf((zi + bi) / cap) : -INFINITY;
    const float fg = ok ? fminf(z, 0.f) - log1pf(expf(-fabsf(z))) : 0.f;
    float F = fg, I = ig;
#pragma unroll
    for (int s = 1; s < 64; s <<= 1) {
      const float Fp = __shfl_up(F, s, 64), Ip = __shfl_up(I, s, 64);
      if (lane >= s) I = fmaxf(Ip + F, I), F += Fp;
    }
    const float mt = fmaxf(F + m, I);
    const float FC = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(F), 63));
    const float mC = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(mt), 63));
    const float gs = ig - F;
    g_af[buf][lane] = (F - mt) * kL2e;
    g_gs[buf][lane] = gs * kL2e;
    g_al[buf][lane] = expf(F + m - mt);
    g_em[buf][lane] = expf(-mt);
    g_w[buf][lane] = expf((FC - mC) + gs);
    m = mC;
  };
  fetch(lo);
  if (wave == 0) {
    fetch_gates(lo);
    make_gates(lo, 0);
  }
  int buf = 0;
  for (int t0 = lo; t0 < hi; t0 += C, buf ^= 1) {
    __syncthreads();                                   // every wave is done with the previous block
    stage();
    __syncthreads();
    const bool more = t0 + C < hi;
    if (more) {
      fetch(t0 + C);
      if (wave == 0) fetch_gates(t0 + C);
    }
    // ---- P for the wave's 16 queries (lane: query 16 wave + col, keys 16 st + 4 grp + i), tiles st <= wave
    f32x4 pacc[4];
#pragma unroll
    for (int st = 0; st < 4; ++st) pacc[st] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kb = 0; kb < NKB; ++kb) {
      const bf16x8 qf = *reinterpret_cast<const bf16x8*>(sq + (16 * wave + col) * QP + 32 * kb + 8 * grp);
#pragma unroll
      for (int st = 0; st < 4; ++st) {
        if (st <= wave) {                              // wave-uniform
          const bf16x8 kf = *reinterpret_cast<const bf16x8*>(sk + (16 * st + col) * QP + 32 * kb + 8 * grp);
          pacc[st] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf, pacc[st], 0, 0, 0);
        }
      }
    }
    // ---- n . q of the state before the block: 4 threads per token
    {
      const int t = tid >> 2, part = tid & 3;
      float a = 0.f;
#pragma unroll
      for (int r = 0; r < NKB; ++r) {
        const int at = part * (DP / 4) + 8 * r;
        const bf16x8 qv = *reinterpret_cast<const bf16x8*>(sq + t * QP + at);
        const f32x4 n0 = *reinterpret_cast<const f32x4*>(sn + at), n1 = *reinterpret_cast<const f32x4*>(sn + at + 4);
#pragma unroll
        for (int j = 0; j < 4; ++j) a = fmaf(bf2f(qv[j]), n0[j], a), a = fmaf(bf2f(qv[4 + j]), n1[j], a);
      }
      a += __shfl_xor(a, 1, 64);
      a += __shfl_xor(a, 2, 64);
      if (part == 0) qn[t] = a * q_scale;
    }
    bf16x4 ph[4], pl[4];
    {
      const int t = 16 * wave + col;
      const float af = g_af[buf][t];
      float sum = 0.f;
#pragma unroll
      for (int st = 0; st < 4; ++st) {
        const f32x4 gs = *reinterpret_cast<const f32x4*>(&g_gs[buf][16 * st + 4 * grp]);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float e = __builtin_amdgcn_exp2f(af + gs[i]);
          const float p = st <= wave && 16 * st + 4 * grp + i <= t ? pacc[st][i] * q_scale * e : 0.f;
          sum += p;
          const uint32_t u = __float_as_uint(p) & 0xffff0000u;
          ph[st][i] = (bf16)__uint_as_float(u);
          pl[st][i] = (bf16)(p - __uint_as_float(u));
        }
      }
      sum = rows_sum(sum);
      if (grp == 0) rs[t] = sum;
    }
    // ---- q S: the accumulators in three bf16 pieces as the B operand
    f32x4 acc[4][CT];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) acc[i][ct] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kb = 0; kb < NKB; ++kb) {
      bf16x8 qa[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) qa[i] = *reinterpret_cast<const bf16x8*>(sq + (16 * i + col) * QP + 32 * kb + 8 * grp);
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        float e[8];
#pragma unroll
        for (int j = 0; j < 4; ++j) e[j] = S[2 * kb][ct][j], e[4 + j] = S[2 * kb + 1][ct][j];
        bf16x8 sp[3];
        ml_split3(e, sp);
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int z = 0; z < 3; ++z) acc[i][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qa[i], sp[z], acc[i][ct], 0, 0, 0);
      }
    }
    if (wave == 0 && more) make_gates(t0 + C, buf ^ 1);
    __syncthreads();                                   // every wave is done with K's rows and with n
    bf16* sph = sk;
    bf16* spl = sk + C * TP;
#pragma unroll
    for (int st = 0; st < 4; ++st) {
      if (st <= (wave | 1)) {                          // the key tiles that the wave's queries read below
        *reinterpret_cast<bf16x4*>(sph + (16 * wave + col) * TP + 16 * st + 4 * grp) = ph[st];
        *reinterpret_cast<bf16x4*>(spl + (16 * wave + col) * TP + 16 * st + 4 * grp) = pl[st];
      }
    }
    const float aC = g_al[buf][C - 1];
    // ---- n <- alpha_C n + sum_s w_s k_s: 2 threads per channel
#pragma unroll
    for (int d0 = 0; d0 < DP; d0 += 128) {
      const int d = d0 + (tid >> 1), half = tid & 1;
      float a = 0.f;
      if (d < DP) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const bf16x8 kv = *reinterpret_cast<const bf16x8*>(skt + d * TP + 32 * half + 8 * r);
          const f32x4 w0 = *reinterpret_cast<const f32x4*>(&g_w[buf][32 * half + 8 * r]);
          const f32x4 w1 = *reinterpret_cast<const f32x4*>(&g_w[buf][32 * half + 8 * r + 4]);
#pragma unroll
          for (int j = 0; j < 4; ++j) a = fmaf(bf2f(kv[j]), w0[j], a), a = fmaf(bf2f(kv[4 + j]), w1[j], a);
        }
      }
      a += __shfl_xor(a, 1, 64);
      if (d < DP && half == 0) {
        float* p = sn + (d & ~31) + ml_quad((d & 31) >> 2) + (d & 3);
        *p = fmaf(aC, *p, a);
      }
    }
    // the rows of q S times alpha_t
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const f32x4 al = *reinterpret_cast<const f32x4*>(&g_al[buf][16 * i + 4 * grp]);
#pragma unroll
      for (int ct = 0; ct < CT; ++ct)
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[i][ct][j] *= al[j] * q_scale;
    }
    __syncthreads();                                   // P, its row sums and n . q are complete
    // ---- P V
    bf16x8 vf[CT][2];
#pragma unroll
    for (int ct = 0; ct < CT; ++ct)
#pragma unroll
      for (int kb = 0; kb < 2; ++kb)
        vf[ct][kb] = *reinterpret_cast<const bf16x8*>(svt + (vbase + 16 * ct + col) * TP + 32 * kb + 8 * grp);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
      for (int kb = 0; kb <= i >> 1; ++kb) {
        const bf16x8 a0 = *reinterpret_cast<const bf16x8*>(sph + (16 * i + col) * TP + 32 * kb + 8 * grp);
        const bf16x8 a1 = *reinterpret_cast<const bf16x8*>(spl + (16 * i + col) * TP + 32 * kb + 8 * grp);
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
          acc[i][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a0, vf[ct][kb], acc[i][ct], 0, 0, 0);
          acc[i][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a1, vf[ct][kb], acc[i][ct], 0, 0, 0);
        }
      }
    }
    // ---- out: lane (column col, tokens 16 i + 4 grp + j)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int tb = 16 * i + 4 * grp;
      const f32x4 al = *reinterpret_cast<const f32x4*>(&g_al[buf][tb]), em = *reinterpret_cast<const f32x4*>(&g_em[buf][tb]);
      const f32x4 r4 = *reinterpret_cast<const f32x4*>(rs + tb), q4 = *reinterpret_cast<const f32x4*>(qn + tb);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float c = 1.0f / (fmaxf(fabsf(fmaf(al[j], q4[j], r4[j])), em[j]) + den_eps);
        const int t = t0 + tb + j;
        if (t < hi) {
#pragma unroll
          for (int ct = 0; ct < CT; ++ct) {
            const int v = col0 + vbase + 16 * ct + col;
            if (v < Dv) o[((size_t)t * H + h) * Dv + v] = acc[i][ct][j] * c;
          }
        }
      }
    }
    // ---- S <- alpha_C S + K^T (w v), w v in three bf16 pieces
#pragma unroll
    for (int rt = 0; rt < NR; ++rt)
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) S[rt][ct] *= aC;
#pragma unroll
    for (int kb = 0; kb < 2; ++kb) {
      const f32x4 w0 = *reinterpret_cast<const f32x4*>(&g_w[buf][32 * kb + 8 * grp]);
      const f32x4 w1 = *reinterpret_cast<const f32x4*>(&g_w[buf][32 * kb + 8 * grp + 4]);
      bf16x8 vp[CT][3];
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        float e[8];
#pragma unroll
        for (int j = 0; j < 4; ++j) e[j] = bf2f(vf[ct][kb][j]) * w0[j], e[4 + j] = bf2f(vf[ct][kb][4 + j]) * w1[j];
        ml_split3(e, vp[ct]);
      }
#pragma unroll
      for (int rt = 0; rt < NR; ++rt) {
        const bf16x8 ka = *reinterpret_cast<const bf16x8*>(skt + (16 * rt + col) * TP + 32 * kb + 8 * grp);
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
#pragma unroll
          for (int z = 0; z < 3; ++z) S[rt][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, vp[ct][z], S[rt][ct], 0, 0, 0);
      }
    }
  }
  // ---- state out
#pragma unroll
  for (int ct = 0; ct < CT; ++ct) {
    const int v = col0 + vbase + 16 * ct + col;
    if (v >= Dv) continue;
    float* row = s_state + (srow * Dv + v) * D;
#pragma unroll
    for (int rt = 0; rt < NR; ++rt) {
      const int d = 16 * rt + 4 * grp;
      if (d < D) *reinterpret_cast<f32x4*>(row + d) = S[rt][ct];
    }
  }
  if (blockIdx.z != 0) return;
  // with several column slices the others may still have to read n and m: they go to a workspace first
  float* nout = nm_ws ? nm_ws + ((size_t)b * H + h) * (D + 1) : n_state + srow * D;
  __syncthreads();
  for (int d = tid; d < D; d += 256) nout[d] = sn[(d & ~31) + ml_quad((d & 31) >> 2) + (d & 3)];
  if (tid == 0) *(nm_ws ? nout + D : m_state + srow) = m;
}

// n and m of a step whose heads ran in several column slices: workspace [seqs, H, D + 1] -> state
__global__ void __launch_bounds__(64) ml_nm_copy_kernel(const float* __restrict__ ws, float* __restrict__ n_state,
                                                        float* __restrict__ m_state, const int32_t* __restrict__ cu,
                                                        const int32_t* __restrict__ slots, int H, int D) {
  const int h = blockIdx.x, b = blockIdx.y;
  if (cu[b + 1] <= cu[b]) return;
  const float* src = ws + ((size_t)b * H + h) * (D + 1);
  const size_t row = (size_t)slots[b] * H + h;
  for (int d = threadIdx.x; d < D; d += 64) n_state[row * D + d] = src[d];
  if (threadIdx.x == 0) m_state[row] = src[D];
}

// Columns per workgroup of ml_chunk for these sizes (64 or 128): the caller's workspace rule is columns < Dv.
int ml_chunk_cols(int seqs, int H, int D, int Dv) {
  return D <= 128 && Dv > 64 && (long)seqs * H * ((Dv + 127) / 128) >= 256 ? 128 : 64;
}

// o [T, H, Dv] float32; proj [T, ld] bf16 with q [H, D] at column qcol, k at kcol, v [H, Dv] at vcol, the gate logits
// [H] at icol / fcol; s_state [slots, H, Dv, D], n_state [slots, H, D], m_state [slots, H] float32; nm_ws: float32
// [seqs, H, D + 1], required when a head's columns take more than one workgroup.
void ml_chunk(uintptr_t o, uintptr_t proj, long ld, int qcol, int kcol, int vcol, int icol, int fcol, uintptr_t i_bias,
              uintptr_t f_bias, float cap, float q_scale, float den_eps, uintptr_t s_state, uintptr_t n_state,
              uintptr_t m_state, uintptr_t nm_ws, uintptr_t cu, uintptr_t positions, uintptr_t slots, int seqs, int H, int D,
              int Dv, uintptr_t stream) {
  if (seqs <= 0) return;
  DLLM_HOST_CHECK(H > 0 && seqs <= 65535 && D > 0 && D <= 256 && D % 8 == 0 && Dv > 0 && Dv % 8 == 0 && cap > 0.f &&
                      ld % 8 == 0 && qcol >= 0 && kcol >= 0 && vcol >= 0 && icol >= 0 && fcol >= 0 && qcol % 8 == 0 &&
                      kcol % 8 == 0 && vcol % 8 == 0,
                  "matrix memory block sizes");
  DLLM_HOST_CHECK(ld >= (long)qcol + (long)H * D && ld >= (long)kcol + (long)H * D && ld >= (long)vcol + (long)H * Dv &&
                      ld >= (long)icol + H && ld >= (long)fcol + H,
                  "matrix memory block columns");
  const int cols = ml_chunk_cols(seqs, H, D, Dv), slices = (Dv + cols - 1) / cols;
  DLLM_HOST_CHECK(o && proj && proj % 16 == 0 && i_bias && f_bias && s_state && s_state % 16 == 0 && n_state && m_state && cu &&
                      positions && slots && slices <= 65535 && (slices == 1 || nm_ws),
                  "matrix memory block arguments");
  hipStream_t s = (hipStream_t)stream;
  float* ws = slices > 1 ? (float*)nm_ws : nullptr;
#define ML_CHUNK(NKB, CT)                                                                                             \
  hipLaunchKernelGGL(HIP_KERNEL_NAME(ml_chunk_kernel<NKB, CT>), dim3(H, seqs, slices), dim3(256), 0, s, (float*)o,    \
                     (const bf16*)proj, ld, qcol, kcol, vcol, icol, fcol, (const float*)i_bias, (const float*)f_bias, \
                     cap, q_scale, den_eps, (float*)s_state, (float*)n_state, (float*)m_state, ws,                    \
                     (const int32_t*)cu, (const int32_t*)positions, (const int32_t*)slots, H, D, Dv)
#define ML_CHUNK_D(CT)                \
  do {                                \
    if (D <= 32) ML_CHUNK(1, CT);     \
    else if (D <= 64) ML_CHUNK(2, CT); \
    else ML_CHUNK(4, CT);             \
  } while (0)
  if (D > 128) ML_CHUNK(8, 1);
  else if (cols == 128) ML_CHUNK_D(2);
  else ML_CHUNK_D(1);
#undef ML_CHUNK_D
#undef ML_CHUNK
  DLLM_HIP_CHECK(hipGetLastError());
  if (ws) {
    hipLaunchKernelGGL(ml_nm_copy_kernel, dim3(H, seqs), dim3(64), 0, s, (const float*)ws, (float*)n_state, (float*)m_state,
                       (const int32_t*)cu, (const int32_t*)slots, H, D);
    DLLM_HIP_CHECK(hipGetLastError());
  }
}

// --------------------------------------------------------------------------- one token per sequence (decode)
// The whole mixer between its projections in one launch, a workgroup per (sequence, head): gates, normaliser, the
// state's step and read-out, the head's output norm (o / rms(o) * w) and the sigmoid gate.  The step is bound by reading
// and writing the state ([Dv][D] float32): L lanes hold a value column, 4 key channels (16 bytes) each, and 8
// columns' loads of a lane are in flight at a time (with few sequences and heads: 16 waves, so that one workgroup
// has its whole state in flight); the read-out sums over the L lanes without LDS (DPP, row swaps).
template <int L>
__device__ __forceinline__ float ml_lanes_sum(float v) {         // over aligned groups of L lanes, result in all
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xb1 /* quad_perm 1 0 3 2 */, 0xf, 0xf, false));
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4e /* quad_perm 2 3 0 1 */, 0xf, 0xf, false));
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x141 /* row_half_mirror */, 0xf, 0xf, false));
  if constexpr (L >= 16)
    v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x140 /* row_mirror */, 0xf, 0xf, false));
  if constexpr (L >= 32) {
    const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  }
  if constexpr (L >= 64) {
    const auto a = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  }
  return v;
}

template <typename T, int L, int NT>
__global__ void __launch_bounds__(NT) ml_step_kernel(
    void* __restrict__ y_, const void* __restrict__ proj_, long ld, int qcol, int kcol, int vcol, int gcol, int icol,
    int fcol, const float* __restrict__ i_bias, const float* __restrict__ f_bias, float cap, float q_scale, float den_eps,
    float* __restrict__ s_state, float* __restrict__ n_state, float* __restrict__ m_state, const void* __restrict__ w_,
    float eps, const int32_t* __restrict__ cu, const int32_t* __restrict__ positions, const int32_t* __restrict__ slots,
    int H, int D, int Dv) {
  constexpr int NG = NT / L, U = NT == 256 ? 8 : 4;    // columns per pass; passes whose loads go out together
  __shared__ float red[16];
  extern __shared__ float so[];                    // the head's read-out [Dv]
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int t = cu[b];
  if (cu[b + 1] <= t) return;
  const int sub = tid & (L - 1), cg = tid / L, d = 4 * sub;
  const bool dok = d < D;
  const T* row = (const T*)proj_ + (size_t)t * ld;
  const size_t srow = (size_t)slots[b] * H + h;
  const bool resume = positions[t] > 0;
  float q[4], k[4], n[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    q[j] = dok ? (float)row[qcol + h * D + d + j] * q_scale : 0.f;
    k[j] = dok ? (float)row[kcol + h * D + d + j] : 0.f;
    n[j] = dok && resume ? n_state[srow * D + d + j] : 0.f;
  }
  const float m0 = resume ? m_state[srow] : 0.f;
  const float ig = cap * tanhf(((float)row[icol + h] + i_bias[h]) / cap);
  const float z = cap * tanhf(((float)row[fcol + h] + f_bias[h]) / cap);
  const float fg = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
  const float mt = fmaxf(fg + m0, ig), a = expf(fg + m0 - mt), wi = expf(ig - mt);
  float p = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    k[j] *= wi;
    n[j] = fmaf(a, n[j], k[j]);
    p = fmaf(n[j], q[j], p);
  }
  const float c = 1.0f / (fmaxf(fabsf(ml_lanes_sum<L>(p)), expf(-mt)) + den_eps);
  float* sb = s_state + srow * Dv * D;
  for (int v0 = 0; v0 < Dv; v0 += NG * U) {
    f32x4 s[U];
    float vv[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int v = v0 + u * NG + cg;
      s[u] = f32x4{0.f, 0.f, 0.f, 0.f}, vv[u] = 0.f;
      if (v < Dv) {
        if (resume && dok) s[u] = *reinterpret_cast<const f32x4*>(sb + (size_t)v * D + d);
        vv[u] = (float)row[vcol + h * Dv + v];
      }
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int v = v0 + u * NG + cg;
      float r = 0.f;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[u][j] = fmaf(a, s[u][j], k[j] * vv[u]);
        r = fmaf(s[u][j], q[j], r);
      }
      r = ml_lanes_sum<L>(r);
      if (v < Dv) {
        if (dok) *reinterpret_cast<f32x4*>(sb + (size_t)v * D + d) = s[u];
        if (sub == 0) so[v] = r * c;
      }
    }
  }
  __syncthreads();                                 // the read-out is complete; every thread has read n and m
  if (cg == 0 && dok) {
#pragma unroll
    for (int j = 0; j < 4; ++j) n_state[srow * D + d + j] = n[j];
  }
  if (tid == 0) m_state[srow] = mt;
  float ss = 0.f;
  for (int v = tid; v < Dv; v += NT) ss += so[v] * so[v];
  const float inv = 1.0f / sqrtf(block_sum(ss, red) / (float)Dv + eps);
  const T* w = (const T*)w_ + (size_t)h * Dv;
  T* y = (T*)y_ + ((size_t)t * H + h) * Dv;
  for (int v = tid; v < Dv; v += NT) {
    const float g = (float)row[gcol + h * Dv + v];
    y[v] = (T)(so[v] * inv * (float)w[v] * (1.0f / (1.0f + expf(-g))));
  }
}

// y [T, H Dv] of the activation type; proj [T, ld] with q, k, v, the output gate g [H, Dv] and the gate logits at their
// columns; w [H Dv] of the activation type; at most one token per sequence.
void ml_step(uintptr_t y, uintptr_t proj, long ld, int qcol, int kcol, int vcol, int gcol, int icol, int fcol,
             uintptr_t i_bias, uintptr_t f_bias, float cap, float q_scale, float den_eps, uintptr_t s_state,
             uintptr_t n_state, uintptr_t m_state, uintptr_t w, float eps, uintptr_t cu, uintptr_t positions,
             uintptr_t slots, int seqs, int max_q_len, int H, int D, int Dv, int f32, uintptr_t stream) {
  if (seqs <= 0) return;
  DLLM_HOST_CHECK(max_q_len == 1 && H > 0 && seqs <= 65535 && D > 0 && D <= 256 && D % 4 == 0 && Dv > 0 && Dv <= 8192 &&
                      cap > 0.f && qcol >= 0 && kcol >= 0 && vcol >= 0 && gcol >= 0 && icol >= 0 && fcol >= 0,
                  "matrix memory step sizes");
  DLLM_HOST_CHECK(ld >= (long)qcol + (long)H * D && ld >= (long)kcol + (long)H * D && ld >= (long)vcol + (long)H * Dv &&
                      ld >= (long)gcol + (long)H * Dv && ld >= (long)icol + H && ld >= (long)fcol + H,
                  "matrix memory step columns");
  DLLM_HOST_CHECK(y && proj && i_bias && f_bias && s_state && s_state % 16 == 0 && n_state && m_state && w && cu && positions &&
                      slots,
                  "matrix memory step arguments");
#define ML_STEP_N(T, L, NT)                                                                                                 \
  hipLaunchKernelGGL(HIP_KERNEL_NAME(ml_step_kernel<T, L, NT>), dim3(H, seqs), dim3(NT), sizeof(float) * (size_t)Dv,    \
                     (hipStream_t)stream, (void*)y, (const void*)proj, ld, qcol, kcol, vcol, gcol, icol, fcol,       \
                     (const float*)i_bias, (const float*)f_bias, cap, q_scale, den_eps, (float*)s_state,             \
                     (float*)n_state, (float*)m_state, (const void*)w, eps, (const int32_t*)cu,                      \
                     (const int32_t*)positions, (const int32_t*)slots, H, D, Dv)
#define ML_STEP(T, L) do { if ((long)H * seqs < 256) ML_STEP_N(T, L, 1024); else ML_STEP_N(T, L, 256); } while (0)
#define ML_STEP_D(T)                 \
  do {                               \
    if (D <= 32) ML_STEP(T, 8);      \
    else if (D <= 64) ML_STEP(T, 16); \
    else if (D <= 128) ML_STEP(T, 32); \
    else ML_STEP(T, 64);             \
  } while (0)
  if (f32) ML_STEP_D(float);
  else ML_STEP_D(bf16);
#undef ML_STEP_D
#undef ML_STEP
#undef ML_STEP_N
  DLLM_HIP_CHECK(hipGetLastError());
}

}  // namespace dllm
