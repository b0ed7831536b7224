// Delta rule of long portions on the fp32 matrix cores
// (v_mfma_f32_16x16x4_f32): the recurrence of seq_delta.hip over chunks of
// up to 64 rows. With G_i the running sum of log decays inside a chunk
// (per key channel, or one number per row where the decay is one per head),
// S0 the state in front of it, and unit rows q_i, k_i:
//
//   (I + L) U = beta V - (beta K~) S0,   K~_i = k_i exp(G_i),
//   L_ij = beta_i sum_d k_id k_jd exp(G_id - G_jd)   (j < i)
//   O  = Q~ S0 + A U,   A_ij = sum_d q_id k_jd exp(G_id - G_jd)  (j <= i)
//   S1 = exp(G_last) S0 + K^ U^,   K^_j = k_j exp(G_last - G_j) as columns
//
//   prepare  one block per (chunk, head), all chunks at once: A, and
//       U0 = (I + L)^-1 beta V, W = (I + L)^-1 beta K~ by forward
//       substitution over 16-row blocks, Q~, K^
//   scan     one block per (sequence, head, 16 value columns), chunk by
//       chunk: U = U0 - W S0, O, S1; the state stays in registers
//   read-out unit RMS, weight and gate of O
//
// Exponents: exp(G_i - G_j) is split at the borders of the 16-row blocks
// into factors whose exponents are sums of log decays, all <= 0, so nothing
// overflows and no sums longer than a block are subtracted. Inside a 16-row block
// exp(c_i - c_7) exp(c_7 - c_j), about its middle row, is used while the
// log decays of either half sum to more than MIN_HALF_LOG (both factors
// finite in fp32). Stronger decays: pairs of different 4-row groups are split
// at the last row of j's group (exponents <= 0 again, one pass per group),
// pairs inside a group about its second row; and where even two rows decay
// past MIN_HALF_LOG, exp(c_i - c_j) is taken per channel, element by element.
// One decay per head needs none of this: exp(G_i - G_j) is a factor of the
// finished product, which is exact in fp32 from the raw bf16 rows
// (v_mfma_f32_16x16x32_bf16); it is summed from the block border on as above.
//
// Fragments: with k = 4 g + e (g = lane / 16) the operand A of four
// consecutive MFMAs is row lane % 16, columns 4 g .. 4 g + 3 of a 16x16 tile
// (one float4 per lane), and the result's layout (rows 4 g + r, column
// lane % 16) is itself the operand B of a following product. The state, U
// and the substitution's columns are therefore never rearranged. Operands
// that another kernel reads are stored tile by tile in lane order.
#include "seq_common.h"

namespace arks {

constexpr int DC = 64;                 // rows per chunk
constexpr int DELTA_CUS = 256;         // compute units of the chip
constexpr float MIN_HALF_LOG = -80.f;  // exp(80) and exp(-80) are finite

__device__ __forceinline__ float4v mm16(float4v acc, float4v a, float4v b) {
#pragma unroll
  for (int e = 0; e < 4; ++e)
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], acc, 0, 0, 0);
  return acc;
}

// log1p(exp(x)) with the hardware exponential and logarithm; log(1 + z) is
// corrected by z / ((1 + z) - 1), which restores the digits 1 + z drops
__device__ __forceinline__ float softplus_fast(float x) {
  const float z = __expf(-fabsf(x));
  const float w = 1.f + z;
  const float d = w - 1.f;
  const float l = d > 0.f ? __logf(w) * (z / d) : z;
  return fmaxf(x, 0.f) + l;
}

struct DeltaChunk {  // float offsets inside the scratch of one (chunk, head)
  int W, Q, K, U, A, E, total;
};
__host__ __device__ inline DeltaChunk delta_chunk_layout(int D, int V) {
  DeltaChunk c;
  c.W = 0;
  c.Q = c.W + DC * D;
  c.K = c.Q + DC * D;
  c.U = c.K + DC * D;
  c.A = c.U + DC * V;
  c.E = c.A + DC * DC;
  c.total = c.E + D;
  return c;
}

// HEAD: one decay per head (a float per row in LDS, not one per channel)
template <bool HEAD>
__host__ __device__ constexpr int delta_prepare_lds(int D) {
  return 2 * DC * (D + 8) * 2 + DC * (HEAD ? 1 : D + 4) * 4 + 10 * 64 * 16 +
         4 * (HEAD ? 1 : D) * 4 + (3 * DC + 8) * 4;
}

typedef __attribute__((ext_vector_type(8))) __bf16 delta_bf16x8;

template <int KT, bool HEAD>
__global__ __launch_bounds__(256, HEAD ? 3 : 2) void delta_chunk_prepare_kernel(
    float* __restrict__ scratch, const bf16* __restrict__ u, int64_t ldu,
    const void* __restrict__ decay_p, int64_t lda,
    const bf16* __restrict__ beta, int64_t ldb, const float* __restrict__ rate,
    const float* __restrict__ dt_bias, const int* __restrict__ cu, int H,
    int G, int V, float unit_eps) {
  constexpr int D = 16 * KT;
  constexpr int LK = D + 8;  // bf16 row stride
  constexpr int LC = HEAD ? 1 : D + 4;  // float row stride
  constexpr int TC = HEAD ? 1 : D;      // decays of a block's totals
  extern __shared__ __align__(16) char smem[];
  bf16* k_s = reinterpret_cast<bf16*>(smem);           // [DC][LK]
  bf16* q_s = k_s + DC * LK;                           // [DC][LK]
  float* c_s = reinterpret_cast<float*>(q_s + DC * LK);  // [DC][LC]
  // L's blocks below the diagonal, then the diagonal ones, which their
  // inverses replace
  float4v* l_s = reinterpret_cast<float4v*>(c_s + DC * LC);  // [6 + 4][64]
  float4v* inv_s = l_s + 6 * 64;                       // [4][64]
  float* tot_s = reinterpret_cast<float*>(l_s + 10 * 64);  // [4][TC]
  float* rk_s = tot_s + 4 * TC;                        // [DC]
  float* rq_s = rk_s + DC;                             // [DC]
  float* b_s = rq_s + DC;                              // [DC]
  float* min_s = b_s + DC;                             // [4]
  float* pair_s = min_s + 4;                           // [4]
  const int h = blockIdx.x, chunk = blockIdx.y;
  const int t0 = cu[chunk], n = min(cu[chunk + 1] - t0, DC);
  const int I = threadIdx.x / 64, lane = threadIdx.x % 64;
  const int g = lane / 16, m = lane % 16;
  const int gk = h / (H / G);
  const DeltaChunk lay = delta_chunk_layout(D, V);
  float* base = scratch + ((int64_t)chunk * H + h) * lay.total;
  // log decays up to a row of its block, and of a whole block
  auto row_log = [&](int row, int d) { return c_s[row * LC + (HEAD ? 0 : d)]; };
  auto block_log = [&](int M, int d) { return tot_s[M * TC + (HEAD ? 0 : d)]; };

  // ---- rows of block I: raw q, k, their unit factors, log decays. Loads
  // are of rows that exist (the last one again past the end) and are not
  // branched around, so that they are all in flight together
  constexpr int DL = (D + 63) / 64;  // channels per lane
  float dec[HEAD ? 1 : DL][HEAD ? 1 : 16];
  if constexpr (HEAD) {
    dec[0][0] = bf16_bits_to_float(reinterpret_cast<const bf16*>(
        decay_p)[(int64_t)(t0 + min(16 * I + m, n - 1)) * lda + h]);
  } else {
    const float* decay = reinterpret_cast<const float*>(decay_p);
#pragma unroll
    for (int j = 0; j < DL; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r)
        dec[j][r] = decay[(int64_t)(t0 + min(16 * I + r, n - 1)) * lda +
                          (int64_t)h * D + min(lane + 64 * j, D - 1)];
  }
  ushort8 qin[4], kin[4];
  const bool live = m * 8 < D;
#pragma unroll
  for (int it = 0; it < 4; ++it) {  // 16 lanes per row
    const bf16* qr = u + (int64_t)(t0 + min(16 * I + 4 * it + g, n - 1)) * ldu +
                     (int64_t)gk * D + min(m * 8, D - 8);
    qin[it] = *reinterpret_cast<const ushort8*>(qr);
    kin[it] = *reinterpret_cast<const ushort8*>(qr + (int64_t)G * D);
  }
#pragma unroll
  for (int it = 0; it < 4; ++it) {
    const int row = 16 * I + 4 * it + g;
    ushort8 qv = qin[it], kv = kin[it];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      qv[e] = live && row < n ? qv[e] : (uint16_t)0;
      kv[e] = live && row < n ? kv[e] : (uint16_t)0;
    }
    float qq = 0.f, kk = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float a = bf16_bits_to_float(qv[e]), b = bf16_bits_to_float(kv[e]);
      qq += a * a;
      kk += b * b;
    }
    qq = group16_reduce_sum(qq);
    kk = group16_reduce_sum(kk);
    if (live) {
      *reinterpret_cast<ushort8*>(q_s + row * LK + m * 8) = qv;
      *reinterpret_cast<ushort8*>(k_s + row * LK + m * 8) = kv;
    }
    if (m == 0) {
      rq_s[row] = 1.f / sqrtf((qq + unit_eps) * (float)D);
      rk_s[row] = 1.f / sqrtf(kk + unit_eps);
    }
  }
  if (lane < 16) {
    const int row = 16 * I + lane;
    b_s[row] = row < n
                   ? sigmoid_f(bf16_bits_to_float(beta[(int64_t)(t0 + row) * ldb + h]))
                   : 0.f;
  }
  if constexpr (HEAD) {
    // running sum over the block's rows, lane m of every 16 lanes has row m
    float c = 16 * I + m < n
                  ? -rate[h] * softplus_fast(dec[0][0] + dt_bias[h]) : 0.f;
#pragma unroll
    for (int off = 1; off < 16; off <<= 1) {
      const float before = __shfl_up(c, off, 16);
      if (m >= off) c += before;
    }
    if (g == 0) {
      c_s[16 * I + m] = c;
      if (m == 15) tot_s[I] = c;
    }
  } else {
    const float rt = rate[h];
    float lowest = 0.f, pair = 0.f;
#pragma unroll
    for (int j = 0; j < DL; ++j) {
      const int d = lane + 64 * j;
      const float db = dt_bias[(int64_t)h * D + min(d, D - 1)];
      float c = 0.f, mid = 0.f, prev2 = 0.f;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const float step = rt * softplus_fast(dec[j][r] + db);
        c -= 16 * I + r < n ? step : 0.f;
        if (d < D) c_s[(16 * I + r) * LC + d] = c;
        if (r == 7) mid = c;
        if (r % 2) {  // two rows' log decay
          pair = fminf(pair, c - prev2);
          prev2 = c;
        }
      }
      if (d < D) tot_s[I * D + d] = c;
      lowest = fminf(lowest, fminf(mid, c - mid));
    }
    lowest = -wave_reduce_max(-lowest);
    pair = -wave_reduce_max(-pair);
    if (lane == 0) {
      min_s[I] = lowest;
      pair_s[I] = pair;
    }
  }
  __syncthreads();

  // ---- scores of block row I against every block J <= I
  if constexpr (HEAD) {
    const int row = 16 * I + m;
    const float rk = rk_s[row], rq = rq_s[row], bI = b_s[row];
    const float ci = c_s[row];
    float pre = 0.f;
    for (int M = 0; M < I; ++M) pre += tot_s[M];
    const float fq = rq * __expf(pre + ci);
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const ushort4v qr =
          *reinterpret_cast<const ushort4v*>(q_s + row * LK + 16 * kt + 4 * g);
      float4v qg;
#pragma unroll
      for (int e = 0; e < 4; ++e) qg[e] = bf16_bits_to_float(qr[e]) * fq;
      *reinterpret_cast<float4v*>(base + lay.Q + ((I * KT + kt) * 64 + lane) * 4) = qg;
    }
    constexpr int STEPS = D / 32;
    delta_bf16x8 kI[STEPS], qI[STEPS];
#pragma unroll
    for (int st = 0; st < STEPS; ++st) {
      kI[st] = *reinterpret_cast<const delta_bf16x8*>(k_s + row * LK + st * 32 + 8 * g);
      qI[st] = *reinterpret_cast<const delta_bf16x8*>(q_s + row * LK + st * 32 + 8 * g);
    }
    float between = 0.f;  // whole blocks between J and I
    for (int J = I; J >= 0; --J) {
      float4v kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int st = 0; st < STEPS; ++st) {
        const delta_bf16x8 a = *reinterpret_cast<const delta_bf16x8*>(
            k_s + (16 * J + m) * LK + st * 32 + 8 * g);
        kk = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, kI[st], kk, 0, 0, 0);
        qk = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, qI[st], qk, 0, 0, 0);
      }
      // lane holds (row i = m of block I, columns j = 4 g + r of block J)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 4 * g + r;
        const float cj = c_s[16 * J + j];
        const float x = J == I ? ci - cj : (tot_s[J] - cj) + between + ci;
        const float f = __expf(fminf(x, 0.f)) * rk_s[16 * J + j];
        kk[r] = J == I && j >= m ? 0.f : kk[r] * f * rk * bI;
        qk[r] = J == I && j > m ? 0.f : qk[r] * f * rq;
      }
      if (J < I) between += tot_s[J];
      l_s[(J == I ? 6 + I : I * (I - 1) / 2 + J) * 64 + lane] = kk;
      *reinterpret_cast<float4v*>(base + lay.A + ((I * 4 + J) * 64 + lane) * 4) = qk;
    }
  } else {
    float4v kI[KT], qI[KT];  // k_i exp(c_i), q_i exp(c_i): row m, 4 channels
    const int row = 16 * I + m;
    const float rk = rk_s[row], rq = rq_s[row];
#pragma unroll
    for (int kt = 0; kt < KT; ++kt) {
      const int d = 16 * kt + 4 * g;
      const ushort4v kr = *reinterpret_cast<const ushort4v*>(k_s + row * LK + d);
      const ushort4v qr = *reinterpret_cast<const ushort4v*>(q_s + row * LK + d);
      const float4v c = *reinterpret_cast<const float4v*>(c_s + row * LC + d);
      float4v qg, pre = {0.f, 0.f, 0.f, 0.f};
      for (int M = 0; M < I; ++M)
        pre += *reinterpret_cast<const float4v*>(tot_s + M * D + d);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float x = __expf(c[e]);
        kI[kt][e] = bf16_bits_to_float(kr[e]) * rk * x;
        qI[kt][e] = bf16_bits_to_float(qr[e]) * rq * x;
        qg[e] = qI[kt][e] * __expf(pre[e]);
      }
      *reinterpret_cast<float4v*>(base + lay.Q + ((I * KT + kt) * 64 + lane) * 4) = qg;
    }
    const float bI = b_s[row];
    const bool split = min_s[I] > MIN_HALF_LOG;
    const bool groups = pair_s[I] > MIN_HALF_LOG;
    for (int J = 0; J <= I; ++J) {
      float4v kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
      const int rj = 16 * J + m;
      const float rkj = rk_s[rj];
      if (J < I) {
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) {
          const int d = 16 * kt + 4 * g;
          const ushort4v kr = *reinterpret_cast<const ushort4v*>(k_s + rj * LK + d);
          float4v x = -*reinterpret_cast<const float4v*>(c_s + rj * LC + d);
          for (int M = J; M < I; ++M)
            x += *reinterpret_cast<const float4v*>(tot_s + M * D + d);
          float4v a;
#pragma unroll
          for (int e = 0; e < 4; ++e)
            a[e] = bf16_bits_to_float(kr[e]) * rkj * __expf(fminf(x[e], 0.f));
          kk = mm16(kk, a, kI[kt]);
          qk = mm16(qk, a, qI[kt]);
        }
      } else if (split) {
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) {
          const int d = 16 * kt + 4 * g;
          const ushort4v kr = *reinterpret_cast<const ushort4v*>(k_s + row * LK + d);
          const ushort4v qr = *reinterpret_cast<const ushort4v*>(q_s + row * LK + d);
          const float4v x = *reinterpret_cast<const float4v*>(c_s + row * LC + d) -
                            *reinterpret_cast<const float4v*>(c_s + (16 * I + 7) * LC + d);
          float4v a, kd, qd;
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float up = __expf(x[e]);
            a[e] = bf16_bits_to_float(kr[e]) * rk * __expf(-x[e]);
            kd[e] = bf16_bits_to_float(kr[e]) * rk * up;
            qd[e] = bf16_bits_to_float(qr[e]) * rq * up;
          }
          kk = mm16(kk, a, kd);
          qk = mm16(qk, a, qd);
        }
      } else if (groups) {
        // lane's row m as i (operand B) and as j (operand A). Pass b < 3:
        // the border behind group b, j in group b, i in a later group; pass
        // 3: i and j of one group about its second row, what it says about
        // other pairs is dropped
        float4v kk3 = {0.f, 0.f, 0.f, 0.f}, qk3 = {0.f, 0.f, 0.f, 0.f};
        const int mg = m / 4;
        for (int b = 0; b < 4; ++b) {
          const int ref = 16 * I + (b < 3 ? 4 * b + 3 : 4 * mg + 1);
          const float use_j = b == 3 || mg == b ? rk : 0.f;
          const float use_i = b == 3 || mg > b ? 1.f : 0.f;
          float4v k1 = {0.f, 0.f, 0.f, 0.f}, q1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int kt = 0; kt < KT; ++kt) {
            const int d = 16 * kt + 4 * g;
            const ushort4v kr = *reinterpret_cast<const ushort4v*>(k_s + row * LK + d);
            const ushort4v qr = *reinterpret_cast<const ushort4v*>(q_s + row * LK + d);
            const float4v x = *reinterpret_cast<const float4v*>(c_s + row * LC + d) -
                              *reinterpret_cast<const float4v*>(c_s + ref * LC + d);
            float4v a, kd, qd;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              // a row that is not used keeps a finite factor
              const float up = use_i * __expf(fminf(x[e], 80.f));
              a[e] = bf16_bits_to_float(kr[e]) * use_j * __expf(fminf(-x[e], 80.f));
              kd[e] = bf16_bits_to_float(kr[e]) * rk * up;
              qd[e] = bf16_bits_to_float(qr[e]) * rq * up;
            }
            k1 = mm16(k1, a, kd);
            q1 = mm16(q1, a, qd);
          }
          if (b < 3) {
            kk += k1;
            qk += q1;
          } else {
            kk3 = k1;
            qk3 = q1;
          }
        }
        // lane holds (i = m, j = 4 g + r): one group where g == m / 4
        if (g == mg) {
          kk = kk3;
          qk = qk3;
        }
      } else {
        // element (i = m, j = 4 g + r) channel by channel
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = 16 * I + 4 * g + r;
          float sk = 0.f, sq = 0.f;
          if (j <= row) {
            for (int d = 0; d < D; ++d) {
              const float x = __expf(fminf(c_s[row * LC + d] - c_s[j * LC + d], 0.f)) *
                              bf16_bits_to_float(k_s[j * LK + d]);
              sk += x * bf16_bits_to_float(k_s[row * LK + d]);
              sq += x * bf16_bits_to_float(q_s[row * LK + d]);
            }
          }
          kk[r] = sk * rk * rk_s[j];
          qk[r] = sq * rq * rk_s[j];
        }
      }
      // lane holds (row i = m of block I, columns j = 4 g + r of block J)
      if (J == I) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = 4 * g + r;
          if (j >= m) kk[r] = 0.f;
          if (j > m) qk[r] = 0.f;
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) kk[r] *= bI;
      l_s[(J == I ? 6 + I : I * (I - 1) / 2 + J) * 64 + lane] = kk;
      *reinterpret_cast<float4v*>(base + lay.A + ((I * 4 + J) * 64 + lane) * 4) = qk;
    }
  }
  __syncthreads();

  // ---- (I + L_II)^-1 of block I, a column per lane (column m)
  {
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float s = i == m ? 1.f : 0.f;
#pragma unroll
      for (int jb = 0; jb < 4; ++jb) {
        if (4 * jb < i) {
          const float4v l = l_s[(6 + I) * 64 + i + 16 * jb];
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (4 * jb + e < i) s -= l[e] * x[4 * jb + e];
        }
      }
      x[i] = s;
    }
    if (g == 0) {
      float* dst = reinterpret_cast<float*>(inv_s + I * 64);
#pragma unroll
      for (int i = 0; i < 16; ++i) dst[(i + 16 * (m / 4)) * 4 + m % 4] = x[i];
    }
  }
  __syncthreads();

  // ---- columns of [K~ | V] through the substitution, 16 at a time
  const int VT = V / 16;
  // q is not needed any more: a 16x16 tile per wave to turn -W's tiles from
  // result layout into operand layout
  float* turn = reinterpret_cast<float*>(q_s) + I * 16 * 20;
  for (int tile = I; tile < KT + VT; tile += 4) {
    const bool is_k = tile < KT;
    const int ct = is_k ? tile : tile - KT;
    const int d = 16 * ct + m;
    float4v X[4], vin[4];
    float pre = 0.f;
    if (!is_k) {
      const bf16* vp = u + (int64_t)t0 * ldu + 2 * (int64_t)G * D + (int64_t)h * V + d;
#pragma unroll
      for (int B = 0; B < 4; ++B)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          vin[B][r] = bf16_bits_to_float(
              vp[(int64_t)min(16 * B + 4 * g + r, n - 1) * ldu]);
    }
#pragma unroll
    for (int B = 0; B < 4; ++B) {
      float4v rhs;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = 16 * B + 4 * g + r;
        float x = 0.f;
        if (is_k) {
          x = bf16_bits_to_float(k_s[row * LK + d]) * rk_s[row] *
              __expf(pre + row_log(row, d));
        } else {
          x = vin[B][r];  // rows past the end have b_s 0
        }
        rhs[r] = x * b_s[row];
      }
      if (is_k) pre += block_log(B, d);
      float4v acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int J = 0; J < 4; ++J)
        if (J < B) acc = mm16(acc, l_s[(B * (B - 1) / 2 + J) * 64 + lane], X[J]);
      rhs -= acc;
      const float4v zero = {0.f, 0.f, 0.f, 0.f};
      X[B] = mm16(zero, inv_s[B * 64 + lane], rhs);
      if (is_k) {
        // within one wave: LDS serves its accesses in order
#pragma unroll
        for (int r = 0; r < 4; ++r) turn[(4 * g + r) * 20 + m] = -X[B][r];
        __builtin_amdgcn_wave_barrier();
        *reinterpret_cast<float4v*>(base + lay.W + ((B * KT + ct) * 64 + lane) * 4) =
            *reinterpret_cast<const float4v*>(turn + m * 20 + 4 * g);
        __builtin_amdgcn_wave_barrier();
      } else {
        *reinterpret_cast<float4v*>(base + lay.U + ((ct * 4 + B) * 64 + lane) * 4) = X[B];
      }
    }
  }

  // ---- K^ transposed (rows = channels) and the chunk's decay
  for (int tile = I; tile < KT * 4; tile += 4) {
    const int rt = tile / 4, kt = tile % 4;
    const int d = 16 * rt + m;
    float post = 0.f;
    for (int M = kt; M < 4; ++M) post += block_log(M, d);
    float4v o;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int j = 16 * kt + 4 * g + e;
      o[e] = bf16_bits_to_float(k_s[j * LK + d]) * rk_s[j] *
             __expf(fminf(post - row_log(j, d), 0.f));
    }
    *reinterpret_cast<float4v*>(base + lay.K + ((rt * 4 + kt) * 64 + lane) * 4) = o;
  }
  for (int d = threadIdx.x; d < D; d += 256)
    base[lay.E + d] = __expf(block_log(0, d) + block_log(1, d) +
                             block_log(2, d) + block_log(3, d));
}

// One block per (sequence, head, NC * 16 value columns); a sequence's chunks
// are DC rows each, the last one what is left. Wave w computes rows
// 16 w .. 16 w + 15 of -W S0, Q~ S0, U and O, and owns the state's 16-row
// tiles w, w + 4, ...; state and U tiles pass between the waves through LDS in
// the layout they have in registers.
template <int KT, int NC>
__global__ __launch_bounds__(256, 2) void delta_chunk_scan_kernel(
    float* __restrict__ o, const float* __restrict__ scratch,
    float* __restrict__ state, const int* __restrict__ chunk_off,
    const int* __restrict__ cu, const int* __restrict__ seq_lens,
    const int* __restrict__ slots, int H, int V, int groups) {
  constexpr int D = 16 * KT;
  constexpr int RT = (KT + 3) / 4;
  __shared__ float4v s_s[NC][KT][64];
  __shared__ float4v u_s[NC][4][64];
  // the column blocks of one (sequence, head) sit on one XCD, whose L2
  // then reads the chunk operands once for all of them
  const int VB = V / (16 * NC);
  const int group = (blockIdx.x / 8 / VB) * 8 + blockIdx.x % 8;
  const int ct = (blockIdx.x / 8) % VB * NC;  // first 16-column tile
  if (group >= groups) return;
  const int s = group / H, h = group % H;
  const int c_begin = chunk_off[s], c_end = chunk_off[s + 1];
  if (c_begin == c_end) return;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x / 64);
  const int lane = threadIdx.x % 64;
  const int g = lane / 16, m = lane % 16;
  const int row0 = cu[s], row_end = cu[s + 1];
  const int start = seq_lens[s] - (row_end - row0);
  const int slot = slots[s];
  float* sp = state + ((int64_t)(slot < 0 ? 0 : slot) * H + h) * D * V + 16 * ct + m;
  const DeltaChunk lay = delta_chunk_layout(D, V);
  const int64_t step = (int64_t)H * lay.total;
  const float* base = scratch + ((int64_t)c_begin * H + h) * lay.total;
  // whether tile w + 4 i exists: known at compile time for whole rounds
  auto mine = [&](int i) { return KT % 4 == 0 || w + 4 * i < KT; };
  const float4v zero = {0.f, 0.f, 0.f, 0.f};
  float4v S[NC][RT];
#pragma unroll
  for (int c = 0; c < NC; ++c)
#pragma unroll
    for (int i = 0; i < RT; ++i) {
      const int rt = w + 4 * i;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        S[c][i][r] = mine(i) && start > 0 && slot >= 0
                         ? sp[(int64_t)(16 * rt + 4 * g + r) * V + 16 * c] : 0.f;
      if (mine(i)) s_s[c][rt][lane] = S[c][i];
    }
  // this wave's operands of one chunk. Each is loaded for the next chunk as
  // soon as its last product has been issued, so that a load has a whole
  // chunk's time and the loads are spread among the products; the scheduling
  // barriers keep them there.
  float4v xw[KT], xq[KT], xk[RT][4], xe[RT], xa[4], xu[NC];
  auto load_wq = [&](const float* b, int kt) {
    xw[kt] = *reinterpret_cast<const float4v*>(b + lay.W + ((w * KT + kt) * 64 + lane) * 4);
    xq[kt] = *reinterpret_cast<const float4v*>(b + lay.Q + ((w * KT + kt) * 64 + lane) * 4);
  };
  auto load_u = [&](const float* b, int c) {
    xu[c] = *reinterpret_cast<const float4v*>(b + lay.U + (((ct + c) * 4 + w) * 64 + lane) * 4);
  };
  auto load_a = [&](const float* b, int J) {
    xa[J] = *reinterpret_cast<const float4v*>(b + lay.A + ((w * 4 + min(J, w)) * 64 + lane) * 4);
  };
  auto load_k = [&](const float* b, int i, int t) {
    if (mine(i))
      xk[i][t] = *reinterpret_cast<const float4v*>(b + lay.K + (((w + 4 * i) * 4 + t) * 64 + lane) * 4);
  };
  auto load_e = [&](const float* b, int i) {
    if (mine(i))
      xe[i] = *reinterpret_cast<const float4v*>(b + lay.E + 16 * (w + 4 * i) + 4 * g);
  };
#pragma unroll
  for (int kt = 0; kt < KT; ++kt) load_wq(base, kt);
#pragma unroll
  for (int c = 0; c < NC; ++c) load_u(base, c);
#pragma unroll
  for (int J = 0; J < 4; ++J) load_a(base, J);
#pragma unroll
  for (int i = 0; i < RT; ++i) {
    load_e(base, i);
#pragma unroll
    for (int t = 0; t < 4; ++t) load_k(base, i, t);
  }
  const int chunks = c_end - c_begin;
  __syncthreads();
  for (int n = 0; n < chunks; ++n) {
    const float* next = base + min(n + 1, chunks - 1) * step;
    // two accumulators per product, so that no MFMA waits for the one
    // before it
    float4v aw[NC][2], aq[NC][2];
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int p = 0; p < 2; ++p) { aw[c][p] = zero; aq[c][p] = zero; }
#pragma unroll
    for (int kt = 0; kt < KT; kt += 2) {
      float4v b[NC][2];
#pragma unroll
      for (int c = 0; c < NC; ++c)
#pragma unroll
        for (int p = 0; p < 2; ++p) b[c][p] = s_s[c][kt + p][lane];
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int p = 0; p < 2; ++p)
#pragma unroll
          for (int c = 0; c < NC; ++c) {
            aw[c][p] = __builtin_amdgcn_mfma_f32_16x16x4f32(xw[kt + p][e], b[c][p][e], aw[c][p], 0, 0, 0);
            aq[c][p] = __builtin_amdgcn_mfma_f32_16x16x4f32(xq[kt + p][e], b[c][p][e], aq[c][p], 0, 0, 0);
          }
      load_wq(next, kt);
      load_wq(next, kt + 1);
      __builtin_amdgcn_sched_barrier(0);
    }
    float4v ow[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      u_s[c][w][lane] = xu[c] + aw[c][0] + aw[c][1];
      ow[c] = aq[c][0] + aq[c][1];
      load_u(next, c);
    }
    __syncthreads();
    float4v ub[NC][4];
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int t = 0; t < 4; ++t) ub[c][t] = u_s[c][t][lane];
#pragma unroll
    for (int i = 0; i < RT; ++i)
      if (mine(i)) {
#pragma unroll
        for (int c = 0; c < NC; ++c) S[c][i] *= xe[i];
        load_e(next, i);
      }
#pragma unroll
    for (int t = 0; t < 4; ++t) {
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int i = 0; i < RT; ++i)
          if (mine(i)) {
#pragma unroll
            for (int c = 0; c < NC; ++c)
              S[c][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(xk[i][t][e], ub[c][t][e], S[c][i], 0, 0, 0);
          }
#pragma unroll
      for (int i = 0; i < RT; ++i) load_k(next, i, t);
      __builtin_amdgcn_sched_barrier(0);
    }
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < RT; ++i)
        if (mine(i)) s_s[c][w + 4 * i][lane] = S[c][i];
    // the rows' own part of O: nobody waits for it
#pragma unroll
    for (int t = 0; t < 4; ++t)
      if (t <= w) {
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
          for (int c = 0; c < NC; ++c)
            ow[c] = __builtin_amdgcn_mfma_f32_16x16x4f32(xa[t][e], ub[c][t][e], ow[c], 0, 0, 0);
      }
#pragma unroll
    for (int J = 0; J < 4; ++J) load_a(next, J);
    const int t0 = row0 + n * DC + 16 * w + 4 * g;
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (t0 + r < row_end)
          o[((int64_t)(t0 + r) * H + h) * V + 16 * (ct + c) + m] = ow[c][r];
    __syncthreads();
  }
  if (slot >= 0) {
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int i = 0; i < RT; ++i)
        if (mine(i)) {
#pragma unroll
          for (int r = 0; r < 4; ++r)
            sp[(int64_t)(16 * (w + 4 * i) + 4 * g + r) * V + 16 * c] = S[c][i][r];
        }
  }
}

// out = o / rms(o) * w * sigmoid(gate), or silu(gate), per head: 16 lanes per (row, head),
// VPL consecutive values per lane and turn (V a multiple of 16 * VPL).
template <int VPL>
__global__ __launch_bounds__(256) void delta_read_out_kernel(
    bf16* __restrict__ out, int64_t ldo, const float* __restrict__ o,
    const void* __restrict__ gate, int64_t ldg, int gate_f32,
    const float* __restrict__ norm_w, float eps, int64_t heads_total, int H,
    int V, int silu_gate) {
  const int64_t i = (int64_t)blockIdx.x * 16 + threadIdx.x / 16;
  const int m = threadIdx.x % 16;
  const bool live = i < heads_total;
  const int64_t t = live ? i / H : 0;
  const int h = live ? (int)(i % H) : 0;
  const float* orow = o + (t * H + h) * V;
  float ss = 0.f;
  for (int v0 = m * VPL; v0 < V; v0 += 16 * VPL) {
#pragma unroll
    for (int e = 0; e < VPL; e += 4) {
      const float4v x = *reinterpret_cast<const float4v*>(orow + v0 + e);
#pragma unroll
      for (int j = 0; j < 4; ++j) ss += x[j] * x[j];
    }
  }
  ss = group16_reduce_sum(ss);
  if (!live) return;
  const float r = 1.f / sqrtf(ss / (float)V + eps);
  const int64_t gat = t * ldg + (int64_t)h * V;
  bf16* dst = out + t * ldo + (int64_t)h * V;
  for (int v0 = m * VPL; v0 < V; v0 += 16 * VPL) {
#pragma unroll
    for (int e = 0; e < VPL; e += 4) {
      const int v = v0 + e;
      const float4v x = *reinterpret_cast<const float4v*>(orow + v);
      const float4v w = *reinterpret_cast<const float4v*>(norm_w + v);
      float gv[4];
      if (gate_f32) {
        const float4v y = *reinterpret_cast<const float4v*>((const float*)gate + gat + v);
#pragma unroll
        for (int j = 0; j < 4; ++j) gv[j] = y[j];
      } else {
        const ushort4v y = *reinterpret_cast<const ushort4v*>((const bf16*)gate + gat + v);
#pragma unroll
        for (int j = 0; j < 4; ++j) gv[j] = bf16_bits_to_float(y[j]);
      }
      ushort4v z;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        z[j] = float_to_bf16_bits(x[j] * r * w[j] * (silu_gate ? gv[j] : 1.f) /
                                  (1.f + __expf(-gv[j])));
      *reinterpret_cast<ushort4v*>(dst + v) = z;
    }
  }
}

template <int KT, bool HEAD>
static void launch_delta_chunks(float* o, float* scratch, const void* u,
                                int64_t ldu, const void* decay, int64_t lda,
                                const void* beta, int64_t ldb, const void* rate,
                                const void* dt_bias, float unit_eps,
                                void* state, const int* chunk_off,
                                const int* chunk_cu, const int* cu,
                                const int* seq_lens, const int* slots,
                                int chunks, int S, int H, int G, int V,
                                hipStream_t stream) {
  constexpr int lds = delta_prepare_lds<HEAD>(16 * KT);
  static bool set = false;
  if (!set) {
    (void)hipFuncSetAttribute(
        reinterpret_cast<const void*>(delta_chunk_prepare_kernel<KT, HEAD>),
        hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    set = true;
  }
  hipLaunchKernelGGL((delta_chunk_prepare_kernel<KT, HEAD>), dim3(H, chunks),
                     dim3(256), lds, stream, scratch, (const bf16*)u, ldu,
                     decay, lda, (const bf16*)beta, ldb,
                     (const float*)rate, (const float*)dt_bias, chunk_cu, H, G,
                     V, unit_eps);
  const int groups = S * H;
  // 32 columns a block (half the operand traffic per column) once that
  // still gives every CU a block
  const int nc = V % 32 == 0 && (int64_t)groups * (V / 32) >= DELTA_CUS ? 2 : 1;
  const dim3 grid((groups + 7) / 8 * 8 * (V / (16 * nc)));
#define SC(NC)                                                               \
  hipLaunchKernelGGL((delta_chunk_scan_kernel<KT, NC>), grid, dim3(256), 0,  \
                     stream, o, scratch, (float*)state, chunk_off, cu,       \
                     seq_lens, slots, H, V, groups)
  if (nc == 2) SC(2);
  else SC(1);
#undef SC
}

}  // namespace arks

using namespace arks;

extern "C" int64_t arks_seq_delta_chunk_floats(int D, int V) {
  return delta_chunk_layout(D, V).total;
}

// 1: sizes, strides or alignment the kernels are not built for.
extern "C" int arks_seq_delta_chunks(
    void* out, int64_t ldo, void* o, void* scratch, const void* u, int64_t ldu,
    const void* decay, int64_t lda, const void* beta, int64_t ldb,
    const void* gate, int64_t ldg, int gate_f32, const void* rate,
    const void* dt_bias, const void* norm_w, float eps, float unit_eps,
    void* state, const void* chunk_off, const void* chunk_cu, const void* cu,
    const void* seq_lens, const void* slots, int64_t T, int chunks, int S,
    int H, int G, int D, int V, int head_decay, int silu_gate,
    hipStream_t stream) {
  if (T == 0 || chunks == 0) return 0;
#define DKH(KT, HEAD)                                                        \
  launch_delta_chunks<KT, HEAD>(                                             \
      (float*)o, (float*)scratch, u, ldu, decay, lda, beta, ldb, rate,       \
      dt_bias, unit_eps, state, (const int*)chunk_off, (const int*)chunk_cu, \
      (const int*)cu, (const int*)seq_lens, (const int*)slots, chunks, S, H, \
      G, V, stream)
#define DK(KT)                                                               \
  do {                                                                       \
    if (head_decay) DKH(KT, true);                                           \
    else DKH(KT, false);                                                     \
  } while (0)
  if (D == 32) DK(2);
  else if (D == 64) DK(4);
  else if (D == 96) DK(6);
  else if (D == 128) DK(8);
  else return 1;
#undef DK
#undef DKH
  const int64_t heads = T * H;
  const unsigned blocks = (unsigned)((heads + 15) / 16);
#define RO(VPL)                                                              \
  hipLaunchKernelGGL((delta_read_out_kernel<VPL>), dim3(blocks), dim3(256),  \
                     0, stream, (bf16*)out, ldo, (const float*)o, gate, ldg, \
                     gate_f32, (const float*)norm_w, eps, heads, H, V, silu_gate)
  if (V % 128 == 0) RO(8);
  else RO(4);
#undef RO
  return 0;
}

extern "C" int arks_seq_delta_chunks_fit(int64_t ldo, int64_t ldu,
                                         int64_t ldg, const void* out,
                                         const void* u, const void* gate,
                                         int D, int V) {
  if (D != 32 && D != 64 && D != 96 && D != 128) return 0;
  if (V % 16 || V > 512) return 0;
  if (ldu % 8 || ldo % 4 || ldg % 4) return 0;
  return (((uintptr_t)u | (uintptr_t)gate) & 15) == 0 &&
         ((uintptr_t)out & 7) == 0;
}
