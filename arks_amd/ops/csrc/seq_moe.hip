// Expert routing and mixing for the layer-list decoders' sparse
// feed-forward (arks_amd/models/feedforward.py GroupedMoE), bf16 or float
// rows.
//
//   moe_route_grouped  scores over all E experts (logits + bias) in fp32, their softmax or
//       (sigmoid) each logit's own sigmoid; experts are cut into
//       `groups` contiguous runs of E/groups. Choices are made by the score
//       plus (optional) a correction per expert: a run's choice score is its
//       highest, or the sum of its two highest (group_top), and only the
//       `keep` best runs stay eligible; the `top` experts with the largest
//       choice scores among those get their scores, without the correction,
//       divided by their sum (+1e-20) unless renorm is off. Ties go to the
//       lower index (groups and experts).
//       matrix (optional, [T, E]): the row's weights at the experts it uses,
//       0 elsewhere; with shared_gate the logits have a column E more, whose
//       sigmoid is the matrix's column E.
//   moe_sort_pairs  (row, expert) pairs in expert order, stable: the row of
//       every sorted place, every pair's place, the pairs per expert
//   moe_mix_rows  out[t] = sum_j w[t][j] * y[row(t, j)], row given, or
//       ids[t][j] * T + t for dense per-expert outputs y [E, T, H].
#include "seq_common.h"

#include <cfloat>

namespace arks {

constexpr int ROUTE_MAX_E = 1024;
constexpr int ROUTE_MAX_K = 32;

// One wave per row.
__global__ __launch_bounds__(64) void moe_route_grouped_kernel(
    float* __restrict__ weights, int* __restrict__ ids,
    const float* __restrict__ logits, int64_t ldl, int E, int top, int groups,
    int keep, int sigmoid, int renorm, float* __restrict__ matrix,
    const float* __restrict__ bias, const float* __restrict__ correction,
    int group_top, int shared_gate) {
  __shared__ float s_s[ROUTE_MAX_E];  // choice scores
  __shared__ float g_s[ROUTE_MAX_E];  // group scores (groups <= E)
  const int t = blockIdx.x, lane = threadIdx.x;
  const float* row = logits + (int64_t)t * ldl;
  const int64_t ldm = E + shared_gate;
  if (sigmoid) {
    for (int e = lane; e < E; e += 64)
      s_s[e] = sigmoid_f(row[e] + (bias ? bias[e] : 0.f));
  } else {
    float m = -FLT_MAX;
    for (int e = lane; e < E; e += 64)
      m = fmaxf(m, row[e] + (bias ? bias[e] : 0.f));
    m = wave_reduce_max(m);
    float sum = 0.f;
    for (int e = lane; e < E; e += 64) {
      const float p = expf(row[e] + (bias ? bias[e] : 0.f) - m);
      s_s[e] = p;
      sum += p;
    }
    sum = wave_reduce_sum(sum);
    __syncthreads();
    const float inv = 1.f / sum;
    for (int e = lane; e < E; e += 64) s_s[e] *= inv;
  }
  if (correction)  // own entries
    for (int e = lane; e < E; e += 64) s_s[e] += correction[e];
  if (matrix) {
    for (int e = lane; e < E; e += 64) matrix[(int64_t)t * ldm + e] = 0.f;
    if (shared_gate && lane == 0)
      matrix[(int64_t)t * ldm + E] = sigmoid_f(row[E]);
  }
  __syncthreads();
  const int per = E / groups;
  for (int gI = lane; gI < groups; gI += 64) {
    float best = -INFINITY, second = -INFINITY;
    for (int i = 0; i < per; ++i) {
      const float v = s_s[gI * per + i];
      second = fmaxf(second, fminf(best, v));
      best = fmaxf(best, v);
    }
    g_s[gI] = group_top > 1 && per > 1 ? best + second : best;
  }
  __syncthreads();
  // the eligible runs: `keep` argmax passes, the others' experts are
  // marked unavailable. +inf marks a chosen run, -inf an expert that cannot
  // be chosen (any more)
  if (keep < groups) {
    for (int r = 0; r < keep; ++r) {
      float best = -INFINITY;
      int bi = groups;
      for (int gI = lane; gI < groups; gI += 64) {
        const float v = g_s[gI] == INFINITY ? -INFINITY : g_s[gI];
        if (v > best || (v == best && gI < bi)) { best = v; bi = gI; }
      }
#pragma unroll
      for (int off = 32; off > 0; off >>= 1) {
        const float ob = __shfl_xor(best, off, 64);
        const int oi = __shfl_xor(bi, off, 64);
        if (ob > best || (ob == best && oi < bi)) { best = ob; bi = oi; }
      }
      __syncthreads();
      if (lane == 0) g_s[min(bi, groups - 1)] = INFINITY;
      __syncthreads();
    }
    for (int e = lane; e < E; e += 64)
      if (g_s[e / per] != INFINITY) s_s[e] = -INFINITY;
    __syncthreads();
  }
  float wsum = 0.f;
  float wk[ROUTE_MAX_K];
  int ik[ROUTE_MAX_K];
  for (int r = 0; r < top; ++r) {
    float best = -INFINITY;
    int bi = E;
    for (int e = lane; e < E; e += 64) {
      const float v = s_s[e];
      if (v > best || (v == best && e < bi)) { best = v; bi = e; }
    }
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
      const float ob = __shfl_xor(best, off, 64);
      const int oi = __shfl_xor(bi, off, 64);
      if (ob > best || (ob == best && oi < bi)) { best = ob; bi = oi; }
    }
    bi = min(bi, E - 1);  // rows of NaNs stay in bounds
    // the score itself: the choice score where there is no correction
    const float sc = !correction ? best
                     : sigmoid   ? sigmoid_f(row[bi] + (bias ? bias[bi] : 0.f))
                                 : best - correction[bi];
    wk[r] = sc;
    ik[r] = bi;
    wsum += sc;
    __syncthreads();
    if (lane == 0) s_s[bi] = -INFINITY;
    __syncthreads();
  }
  if (lane == 0) {
    const float d = wsum + 1e-20f;
    for (int r = 0; r < top; ++r) {
      const float w = renorm ? wk[r] / d : wk[r];
      weights[(int64_t)t * top + r] = w;
      ids[(int64_t)t * top + r] = ik[r];
      if (matrix) matrix[(int64_t)t * ldm + ik[r]] = w;
    }
  }
}

// Stable counting sort in one block. Wave w owns the w-th run of pairs; its
// pairs of expert e go to a run of places of their own, in order: a lane's
// place inside a group of 64 pairs is the number of lower lanes with the same
// expert, found by intersecting ballots of the expert's bits.
constexpr int SORT_WAVES = 16;
constexpr int SORT_MAX_E = 512;

__global__ __launch_bounds__(64 * SORT_WAVES) void moe_sort_pairs_kernel(
    int* __restrict__ row_of_place, int* __restrict__ place,
    int* __restrict__ counts, const int* __restrict__ ids, int n, int k, int E,
    int pad) {
  extern __shared__ int at_s[];  // [SORT_WAVES][E]: next free place
  __shared__ int first_s[SORT_MAX_E];
  const int w = threadIdx.x / 64, lane = threadIdx.x % 64;
  const int per = (n + SORT_WAVES * 64 - 1) / (SORT_WAVES * 64) * 64;
  const int lo = min(w * per, n), hi = min(lo + per, n);
  for (int i = threadIdx.x; i < SORT_WAVES * E; i += blockDim.x) at_s[i] = 0;
  for (int i = threadIdx.x; i < pad; i += blockDim.x) row_of_place[n + i] = 0;
  __syncthreads();
  for (int i = lo + lane; i < hi; i += 64) atomicAdd(&at_s[w * E + ids[i]], 1);
  __syncthreads();
  for (int e = threadIdx.x; e < E; e += blockDim.x) {
    int sum = 0;
    for (int v = 0; v < SORT_WAVES; ++v) {
      const int c = at_s[v * E + e];
      at_s[v * E + e] = sum;
      sum += c;
    }
    counts[e] = sum;
    first_s[e] = sum;
  }
  __syncthreads();
  if (w == 0) {  // exclusive sum over the experts, 64 at a time
    int before = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int c = e0 + lane < E ? first_s[e0 + lane] : 0;
      int sum = c;
#pragma unroll
      for (int off = 1; off < 64; off <<= 1) {
        const int v = __shfl_up(sum, off, 64);
        if (lane >= off) sum += v;
      }
      if (e0 + lane < E) first_s[e0 + lane] = before + sum - c;
      before += __shfl(sum, 63, 64);
    }
  }
  __syncthreads();
  const int bits = 32 - __clz(max(E - 1, 1));
  volatile int* next_s = at_s + w * E;  // written by other lanes of the wave
  for (int i0 = lo; i0 < hi; i0 += 64) {
    const int i = i0 + lane;
    const bool live = i < hi;
    const int e = live ? ids[i] : 0;
    unsigned long long same = __ballot(live);
    for (int b = 0; b < bits; ++b) {
      const unsigned long long set = __ballot(live && ((e >> b) & 1));
      same &= (e >> b) & 1 ? set : ~set;
    }
    if (live) {
      const int rank = __popcll(same & ((1ull << lane) - 1));
      const int used = next_s[e];
      const int p = first_s[e] + used + rank;
      row_of_place[p] = i / k;
      place[i] = p;
      // the group's last lane moves the run on; lanes of one wave, so all of
      // them have read the old value
      if ((same >> lane) == 1ull) next_s[e] = used + rank + 1;
    }
    __builtin_amdgcn_wave_barrier();
  }
}

template <typename AT>
__global__ __launch_bounds__(256) void moe_mix_rows_kernel(
    AT* __restrict__ out, const AT* __restrict__ y,
    const float* __restrict__ weights, const int* __restrict__ rows, int T,
    int H, int k, int dense, const AT* __restrict__ add) {
  const int t = blockIdx.x;
  for (int c = threadIdx.x; c < H; c += 256) {
    float acc = add ? Act<AT>::ld(add + (int64_t)t * H + c) : 0.f;
    for (int j = 0; j < k; ++j) {
      const int64_t r = dense ? (int64_t)rows[t * k + j] * T + t
                              : (int64_t)rows[t * k + j];
      acc += weights[t * k + j] * Act<AT>::ld(y + r * H + c);
    }
    Act<AT>::st(out + (int64_t)t * H + c, acc);
  }
}

// bf16, 8 channels per thread (H % 8 == 0)
__global__ __launch_bounds__(256) void moe_mix_rows_vec8_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ y,
    const float* __restrict__ weights, const int* __restrict__ rows, int T,
    int H, int k, int dense, const bf16* __restrict__ add) {
  const int t = blockIdx.x;
  for (int c = threadIdx.x * 8; c < H; c += 256 * 8) {
    float acc[8];
    if (add) {
      const ushort8 u = *reinterpret_cast<const ushort8*>(add + (int64_t)t * H + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] = bf16_bits_to_float(u[e]);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] = 0.f;
    }
    for (int j = 0; j < k; ++j) {
      const int64_t r = dense ? (int64_t)rows[t * k + j] * T + t
                              : (int64_t)rows[t * k + j];
      const float w = weights[t * k + j];
      const ushort8 u = *reinterpret_cast<const ushort8*>(y + r * H + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] += w * bf16_bits_to_float(u[e]);
    }
    ushort8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = float_to_bf16_bits(acc[e]);
    *reinterpret_cast<ushort8*>(out + (int64_t)t * H + c) = o;
  }
}

}  // namespace arks

using namespace arks;

extern "C" int arks_seq_moe_route_grouped(void* weights, void* ids,
                                          const void* logits, int64_t ldl,
                                          int T, int E, int top, int groups,
                                          int keep, int sigmoid, int renorm,
                                          void* matrix, const void* bias,
                                          const void* correction,
                                          int group_top, int shared_gate,
                                          hipStream_t stream) {
  if (E > ROUTE_MAX_E || top > ROUTE_MAX_K || groups < 1 || E % groups ||
      keep > groups || top > keep * (E / groups))
    return 1;
  if (T == 0) return 0;
  hipLaunchKernelGGL(moe_route_grouped_kernel, dim3(T), dim3(64), 0, stream,
                     (float*)weights, (int*)ids, (const float*)logits, ldl, E,
                     top, groups, keep, sigmoid, renorm, (float*)matrix,
                     (const float*)bias, (const float*)correction, group_top,
                     shared_gate);
  return 0;
}

// ids are trusted to be in [0, E): they come from the routing kernel.
extern "C" int arks_seq_moe_sort_pairs(void* row_of_place, void* place,
                                       void* counts, const void* ids, int n,
                                       int k, int E, int pad,
                                       hipStream_t stream) {
  if (E > SORT_MAX_E || E < 1 || k < 1) return 1;
  hipLaunchKernelGGL(moe_sort_pairs_kernel, dim3(1), dim3(64 * SORT_WAVES),
                     SORT_WAVES * E * sizeof(int), stream, (int*)row_of_place,
                     (int*)place, (int*)counts, (const int*)ids, n, k, E, pad);
  return 0;
}

extern "C" void arks_seq_moe_mix_rows(void* out, const void* y,
                                      const void* weights, const void* rows,
                                      int T, int H, int k, int dense,
                                      const void* add, int act_f32,
                                      hipStream_t stream) {
  if (T == 0) return;
  if (!act_f32 && H % 8 == 0) {
    hipLaunchKernelGGL(moe_mix_rows_vec8_kernel, dim3(T), dim3(256), 0, stream,
                       (bf16*)out, (const bf16*)y, (const float*)weights,
                       (const int*)rows, T, H, k, dense, (const bf16*)add);
    return;
  }
  SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
      (moe_mix_rows_kernel<AT>), dim3(T), dim3(256), 0, stream, (AT*)out,
      (const AT*)y, (const float*)weights, (const int*)rows, T, H, k, dense,
      (const AT*)add));
}
