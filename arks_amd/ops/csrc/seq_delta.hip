// Delta rule with a decay per head and key channel, or one per head
// (arks_amd/models/mixers.py ChannelDeltaMixer, HeadDeltaMixer), row by row,
// any head sizes, bf16 or float rows, fp32 arithmetic: per head, with
// unit-length q and k (q times D^-1/2), g = exp(-rate softplus(decay +
// dt_bias)) per key channel (or the same for all of them) and b =
// sigmoid(beta),
//   S <- g S,  w = b (v - S^T k),  S <- S + k w^T,  o = S^T q,
// then o at unit RMS over the head, times the norm weight, times
// sigmoid(gate) or silu(gate). With s = g S from the same pass, S^T q after
// the update is s^T q + (k . q) w, so one pass over the state serves both
// products.
//
// One block per (sequence, head). A wave owns CPW = 64 / NRG value columns;
// its lanes are NRG groups of state rows x CPW columns, RPT rows of one
// column in registers per lane, so the two dot products are reduced by
// shuffles inside the wave and waves meet only where a batch of rows is
// staged in LDS (unit q, k, decays, v) and where its outputs are normed.
// Columns beyond the block's waves are walked in turns, the state passing
// through memory between the batches.
#include "seq_common.h"

namespace arks {

struct DeltaDims {
  int H, G, D, V, BR;  // BR: rows staged at a time
  int64_t ldo, ldu, lda, ldb, ldg;
  int gate_f32;
  float eps, unit_eps;
  // head_decay: decay [T, H] in the rows' type and dt_bias [H] instead of
  // float [T, H * D] and [H * D]
  int head_decay, silu_gate;
};

template <typename AT>
__device__ __forceinline__ float delta_decay(const void* decay,
                                             const float* dt_bias, int64_t t,
                                             int h, int d, float rate,
                                             const DeltaDims& a) {
  const float z =
      a.head_decay
          ? Act<AT>::ld(reinterpret_cast<const AT*>(decay) + t * a.lda + h) +
                dt_bias[h]
          : reinterpret_cast<const float*>(decay)[t * a.lda +
                                                  (int64_t)h * a.D + d] +
                dt_bias[(int64_t)h * a.D + d];
  return expf(-rate * softplus_f(z));
}

__device__ __forceinline__ float delta_gate(float z, const DeltaDims& a) {
  const float s = sigmoid_f(z);
  return a.silu_gate ? z * s : s;
}

template <typename AT, int RPT, int NRG>
__global__ __launch_bounds__(512) void channel_delta_scan_kernel(
    AT* __restrict__ out, const AT* __restrict__ u,
    const void* __restrict__ decay, const AT* __restrict__ beta,
    const void* __restrict__ gate, const float* __restrict__ rate,
    const float* __restrict__ dt_bias, const float* __restrict__ norm_w,
    float* __restrict__ state, const int* __restrict__ cu,
    const int* __restrict__ seq_lens, const int* __restrict__ slots,
    DeltaDims a) {
  constexpr int CPW = 64 / NRG;
  constexpr int GS = RPT + 4;     // a row group's stride in LDS
  constexpr int RS = NRG * GS;    // a staged row's stride
  extern __shared__ __align__(16) float smem[];
  const int h = blockIdx.x, s = blockIdx.y;
  const int r0 = cu[s], rows = cu[s + 1] - r0;
  if (rows == 0) return;
  const int D = a.D, V = a.V, BR = a.BR;
  float* k_s = smem;               // [BR][RS]
  float* q_s = k_s + BR * RS;      // [BR][RS]
  float* g_s = q_s + BR * RS;      // [BR][RS]
  float* v_s = g_s + BR * RS;      // [BR][V]
  float* o_s = v_s + BR * V;       // [BR][V]
  float* b_s = o_s + BR * V;       // [BR]
  float* kq_s = b_s + BR;          // [BR]
  const int nthr = blockDim.x, nw = nthr / 64;
  const int wave = threadIdx.x / 64, lane = threadIdx.x % 64;
  const int rg = lane / CPW, col = lane % CPW;
  const int start = seq_lens[s] - rows;
  const int slot = slots[s];
  float* sp = state + ((int64_t)(slot < 0 ? 0 : slot) * a.H + h) * D * V;
  const int gk = h / (a.H / a.G);
  const int ntiles = (V + CPW - 1) / CPW;
  const bool resident = ntiles <= nw;
  const float rt = rate[h];
  const float qmul = 1.f / sqrtf((float)D);
  float S[RPT];
  auto load_state = [&](int tile, bool have) {
    const int v = tile * CPW + col;
    have = have && v < V;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
      const int d = rg * RPT + i;
      S[i] = have && d < D ? sp[(int64_t)d * V + v] : 0.f;
    }
  };
  // in flight while the first rows are staged
  if (resident) load_state(wave, start > 0 && slot >= 0);

  for (int b0 = 0; b0 < rows; b0 += BR) {
    const int nb = min(BR, rows - b0);
    if (b0) __syncthreads();  // the previous batch's readers are done
    // ---- stage: a wave per row
    for (int r = wave; r < nb; r += nw) {
      const int64_t t = r0 + b0 + r;
      const AT* qr = u + t * a.ldu + (int64_t)gk * D;
      const AT* kr = qr + (int64_t)a.G * D;
      float qq = 0.f, kk = 0.f, kq = 0.f;
      for (int d = lane; d < D; d += 64) {
        const float qv = Act<AT>::ld(qr + d), kv = Act<AT>::ld(kr + d);
        qq += qv * qv;
        kk += kv * kv;
        kq += qv * kv;
      }
      qq = wave_reduce_sum(qq);
      kk = wave_reduce_sum(kk);
      kq = wave_reduce_sum(kq);
      const float rq = qmul / sqrtf(qq + a.unit_eps);
      const float rk = 1.f / sqrtf(kk + a.unit_eps);
      for (int d = lane; d < NRG * RPT; d += 64) {
        const int at = r * RS + (d / RPT) * GS + d % RPT;
        float qv = 0.f, kv = 0.f, gv = 1.f;
        if (d < D) {
          qv = Act<AT>::ld(qr + d) * rq;
          kv = Act<AT>::ld(kr + d) * rk;
          gv = delta_decay<AT>(decay, dt_bias, t, h, d, rt, a);
        }
        q_s[at] = qv;
        k_s[at] = kv;
        g_s[at] = gv;
      }
      const AT* vr = u + t * a.ldu + 2 * (int64_t)a.G * D + (int64_t)h * V;
      for (int v = lane; v < V; v += 64) v_s[r * V + v] = Act<AT>::ld(vr + v);
      if (lane == 0) {
        b_s[r] = sigmoid_f(Act<AT>::ld(beta + t * a.ldb + h));
        kq_s[r] = kq * rq * rk;
      }
    }
    __syncthreads();
    // ---- the recurrence
    for (int tile = wave; tile < ntiles; tile += nw) {
      const int v = tile * CPW + col;
      const bool live = v < V;
      if (!resident) load_state(tile, b0 ? slot >= 0 : start > 0 && slot >= 0);
      for (int r = 0; r < nb; ++r) {
        const float4v* kp = reinterpret_cast<const float4v*>(k_s + r * RS + rg * GS);
        const float4v* qp = reinterpret_cast<const float4v*>(q_s + r * RS + rg * GS);
        const float4v* gp = reinterpret_cast<const float4v*>(g_s + r * RS + rg * GS);
        float sk = 0.f, sq = 0.f;
#pragma unroll
        for (int i = 0; i < RPT / 4; ++i) {
          const float4v kv = kp[i], qv = qp[i], gv = gp[i];
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float x = S[4 * i + e] * gv[e];
            S[4 * i + e] = x;
            sk += x * kv[e];
            sq += x * qv[e];
          }
        }
#pragma unroll
        for (int off = CPW; off < 64; off <<= 1) {
          sk += __shfl_xor(sk, off, 64);
          sq += __shfl_xor(sq, off, 64);
        }
        const float w = live ? b_s[r] * (v_s[r * V + v] - sk) : 0.f;
#pragma unroll
        for (int i = 0; i < RPT / 4; ++i) {
          const float4v kv = kp[i];
#pragma unroll
          for (int e = 0; e < 4; ++e) S[4 * i + e] += kv[e] * w;
        }
        if (live && rg == 0) o_s[r * V + v] = sq + kq_s[r] * w;
      }
      if (slot >= 0 && live && (b0 + nb == rows || !resident)) {
#pragma unroll
        for (int i = 0; i < RPT; ++i) {
          const int d = rg * RPT + i;
          if (d < D) sp[(int64_t)d * V + v] = S[i];
        }
      }
    }
    __syncthreads();
    // ---- read-out: unit RMS, weight, gate; a wave per row
    for (int r = wave; r < nb; r += nw) {
      const int64_t t = r0 + b0 + r;
      float ss = 0.f;
      for (int v = lane; v < V; v += 64) ss += o_s[r * V + v] * o_s[r * V + v];
      ss = wave_reduce_sum(ss);
      const float ro = 1.f / sqrtf(ss / (float)V + a.eps);
      const int64_t gat = t * a.ldg + (int64_t)h * V;
      AT* orow = out + t * a.ldo + (int64_t)h * V;
      for (int v = lane; v < V; v += 64) {
        const float gv = a.gate_f32
                             ? reinterpret_cast<const float*>(gate)[gat + v]
                             : Act<AT>::ld(reinterpret_cast<const AT*>(gate) + gat + v);
        Act<AT>::st(orow + v, o_s[r * V + v] * ro * norm_w[v] * delta_gate(gv, a));
      }
    }
  }
}

// Steps that bring one row per sequence: the whole head in one pass, one block
// per (sequence, head), a wave per 32 value columns. 8 lanes x 4 columns read
// 128 bytes of a state row, 8 lane groups take every eighth row, and all of
// the state's loads are in flight while q, k and the decays are prepared.
template <typename AT, int NI>
__global__ __launch_bounds__(512) void channel_delta_step_kernel(
    AT* __restrict__ out, const AT* __restrict__ u,
    const void* __restrict__ decay, const AT* __restrict__ beta,
    const void* __restrict__ gate, const float* __restrict__ rate,
    const float* __restrict__ dt_bias, const float* __restrict__ norm_w,
    float* __restrict__ state, const int* __restrict__ cu,
    const int* __restrict__ seq_lens, const int* __restrict__ slots,
    DeltaDims a) {
  __shared__ float q_s[8 * NI], k_s[8 * NI], g_s[8 * NI];
  __shared__ float red_s[8][3];
  __shared__ float ss_s[8];
  const int h = blockIdx.x, s = blockIdx.y;
  const int D = a.D, V = a.V;
  const int nw = blockDim.x / 64, wave = threadIdx.x / 64, lane = threadIdx.x % 64;
  const int rg = lane / 8;
  const int v = (wave * 8 + lane % 8) * 4;
  const bool live = v < V;
  const int64_t t = cu[s];
  const int slot = slots[s];
  const bool have = live && seq_lens[s] > 1 && slot >= 0;
  float* sp = state + ((int64_t)(slot < 0 ? 0 : slot) * a.H + h) * D * V + v;
  float4v S[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int d = rg + 8 * i;
    S[i] = float4v{0.f, 0.f, 0.f, 0.f};
    if (have && d < D)
      S[i] = *reinterpret_cast<const float4v*>(sp + (int64_t)d * V);
  }
  const AT* qr = u + t * a.ldu + (int64_t)(h / (a.H / a.G)) * D;
  const AT* kr = qr + (int64_t)a.G * D;
  float qq = 0.f, kk = 0.f, kq = 0.f;
  for (int d = threadIdx.x; d < 8 * NI; d += blockDim.x) {
    float qv = 0.f, kv = 0.f, gv = 0.f;
    if (d < D) {
      qv = Act<AT>::ld(qr + d);
      kv = Act<AT>::ld(kr + d);
      gv = delta_decay<AT>(decay, dt_bias, t, h, d, rate[h], a);
    }
    q_s[d] = qv;
    k_s[d] = kv;
    g_s[d] = gv;
    qq += qv * qv;
    kk += kv * kv;
    kq += qv * kv;
  }
  qq = wave_reduce_sum(qq);
  kk = wave_reduce_sum(kk);
  kq = wave_reduce_sum(kq);
  if (lane == 0) {
    red_s[wave][0] = qq;
    red_s[wave][1] = kk;
    red_s[wave][2] = kq;
  }
  __syncthreads();
  qq = kk = kq = 0.f;
  for (int w = 0; w < nw; ++w) {
    qq += red_s[w][0];
    kk += red_s[w][1];
    kq += red_s[w][2];
  }
  const float rq = 1.f / sqrtf((qq + a.unit_eps) * (float)D);
  const float rk = 1.f / sqrtf(kk + a.unit_eps);
  float4v sk = {0.f, 0.f, 0.f, 0.f}, sq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int d = rg + 8 * i;
    S[i] *= g_s[d];
    sk += S[i] * k_s[d];
    sq += S[i] * q_s[d];
  }
#pragma unroll
  for (int off = 8; off < 64; off <<= 1) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      sk[e] += __shfl_xor(sk[e], off, 64);
      sq[e] += __shfl_xor(sq[e], off, 64);
    }
  }
  const float b = sigmoid_f(Act<AT>::ld(beta + t * a.ldb + h));
  const AT* vr = u + t * a.ldu + 2 * (int64_t)a.G * D + (int64_t)h * V + v;
  float4v w, o;
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    const float vv = live ? Act<AT>::ld(vr + e) : 0.f;
    w[e] = b * (vv - sk[e] * rk);
    o[e] = sq[e] * rq + kq * rq * rk * w[e];
    ss += o[e] * o[e];
  }
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int d = rg + 8 * i;
    S[i] += w * (k_s[d] * rk);
    if (live && slot >= 0 && d < D)
      *reinterpret_cast<float4v*>(sp + (int64_t)d * V) = S[i];
  }
#pragma unroll
  for (int off = 1; off < 8; off <<= 1) ss += __shfl_xor(ss, off, 64);
  if (lane == 0) ss_s[wave] = live ? ss : 0.f;
  __syncthreads();
  ss = 0.f;
  for (int i = 0; i < nw; ++i) ss += ss_s[i];
  if (rg == 0 && live) {
    const float ro = 1.f / sqrtf(ss / (float)V + a.eps);
    const int64_t gat = t * a.ldg + (int64_t)h * V + v;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float gv = a.gate_f32
                           ? reinterpret_cast<const float*>(gate)[gat + e]
                           : Act<AT>::ld(reinterpret_cast<const AT*>(gate) + gat + e);
      Act<AT>::st(out + t * a.ldo + (int64_t)h * V + v + e,
                  o[e] * ro * norm_w[v + e] * delta_gate(gv, a));
    }
  }
}

template <typename AT, int RPT, int NRG>
static int launch_delta_scan(void* out, const void* u, const void* decay,
                             const void* beta, const void* gate,
                             const void* rate, const void* dt_bias,
                             const void* norm_w, void* state, const void* cu,
                             const void* seq_lens, const void* slots, int S,
                             int max_rows, DeltaDims a, hipStream_t stream) {
  constexpr int CPW = 64 / NRG;
  const int ntiles = (a.V + CPW - 1) / CPW;
  const int nw = ntiles < 8 ? ntiles : 8;
  const int row_floats = 3 * NRG * (RPT + 4) + 2 * a.V + 2;
  int br = (60 * 1024 / 4) / row_floats;
  if (br < 1) return 1;
  const int want = max_rows > 0 && max_rows < 16 ? max_rows : 16;
  a.BR = br < want ? br : want;
  const size_t lds = (size_t)a.BR * row_floats * 4;
  hipLaunchKernelGGL((channel_delta_scan_kernel<AT, RPT, NRG>), dim3(a.H, S),
                     dim3(nw * 64), lds, stream, (AT*)out, (const AT*)u,
                     decay, (const AT*)beta, gate,
                     (const float*)rate, (const float*)dt_bias,
                     (const float*)norm_w, (float*)state, (const int*)cu,
                     (const int*)seq_lens, (const int*)slots, a);
  return 0;
}

}  // namespace arks

using namespace arks;

extern "C" int arks_seq_channel_delta_scan(
    void* out, int64_t ldo, const void* u, int64_t ldu, const void* decay,
    int64_t lda, const void* beta, int64_t ldb, const void* gate, int64_t ldg,
    int gate_f32, const void* rate, const void* dt_bias, const void* norm_w,
    float eps, float unit_eps, void* state, const void* cu,
    const void* seq_lens, const void* slots, int S, int H, int G, int D, int V,
    int max_rows, int one_row, int head_decay, int silu_gate, int act_f32,
    hipStream_t stream) {
  if (S == 0 || H == 0) return 0;
  const DeltaDims a{H, G, D, V, 0, ldo, ldu, lda, ldb, ldg, gate_f32, eps,
                    unit_eps, head_decay, silu_gate};
  if (max_rows == 1 && one_row && V % 4 == 0 && V <= 256 && D <= 128) {
#define DT(NI)                                                                \
  SEQ_DISPATCH_ACT(act_f32, {                                                 \
    hipLaunchKernelGGL((channel_delta_step_kernel<AT, NI>), dim3(H, S),       \
                       dim3((V + 31) / 32 * 64), 0, stream, (AT*)out,         \
                       (const AT*)u, decay, (const AT*)beta,                  \
                       gate, (const float*)rate, (const float*)dt_bias,       \
                       (const float*)norm_w, (float*)state, (const int*)cu,   \
                       (const int*)seq_lens, (const int*)slots, a);           \
    return 0;                                                                 \
  })
    if (D <= 32) DT(4);
    if (D <= 64) DT(8);
    if (D <= 96) DT(12);
    DT(16);
#undef DT
  }
#define DS(RPT, NRG)                                                          \
  SEQ_DISPATCH_ACT(act_f32, return (launch_delta_scan<AT, RPT, NRG>(          \
      out, u, decay, beta, gate, rate, dt_bias, norm_w, state, cu, seq_lens,  \
      slots, S, max_rows, a, stream)))
  if (D <= 32) DS(8, 4);
  if (D <= 64) DS(16, 4);
  if (D <= 128) DS(32, 4);
  if (D <= 256) DS(32, 8);
  if (D <= 512) DS(32, 16);
#undef DS
  return 1;
}
