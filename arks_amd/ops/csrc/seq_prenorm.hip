// Row kernels of the pre-norm two-mixer blocks (arks_amd/models/hybrid.py
// PreNormBlock), bf16 or float rows, fp32 arithmetic:
//
//   hashed_embed  x = embed[token] * scale + table[row] as the fp32 residual,
//       row = (previous token * mul_prev + token * mul_cur) mod buckets, the
//       table's row `buckets` at a sequence's first position. The previous
//       token of a portion's first row is per-sequence state.
//   row_norm_qk_cache  q and k normed over ALL their heads at once (RMS,
//       a weight per element), q times a factor that grows with the logarithm
//       of the position; k and v to their pages
//   relu_square   max(x, 0)^2
#include "seq_common.h"

namespace arks {

struct HashDims {
  int64_t mul_prev, mul_cur, buckets;
  float scale;
  int W;
};

// Table row of row t. single: every sequence brings one row, so this block
// alone reads the sequence's state and may replace it (once all its threads
// have read it).
__device__ __forceinline__ int64_t hashed_row(
    int t, const int64_t* ids, int* prev, const int* cu, const int* seq_lens,
    const int* slots, const int* token_seq, const HashDims& a, int single) {
  const SeqRow r = seq_row(t, token_seq, cu, seq_lens, slots);
  const int i = t - r.first_row;
  int64_t before = -1;
  if (i > 0) before = ids[t - 1];
  else if (r.start > 0 && r.slot >= 0) before = prev[r.slot];
  if (single) {
    __syncthreads();
    if (threadIdx.x == 0 && r.slot >= 0) prev[r.slot] = (int)ids[t];
  }
  if (before < 0) return a.buckets;
  return (before * a.mul_prev + ids[t] * a.mul_cur) % a.buckets;
}

template <typename AT>
__global__ __launch_bounds__(256) void hashed_embed_kernel(
    float* __restrict__ x, const int64_t* __restrict__ ids,
    const AT* __restrict__ embed, const AT* __restrict__ table, int* prev,
    const int* __restrict__ cu, const int* __restrict__ seq_lens,
    const int* __restrict__ slots, const int* __restrict__ token_seq,
    HashDims a, int single) {
  const int t = blockIdx.x;
  const int64_t row =
      hashed_row(t, ids, prev, cu, seq_lens, slots, token_seq, a, single);
  const AT* e = embed + ids[t] * a.W;
  const AT* b = table + row * a.W;
  for (int c = threadIdx.x; c < a.W; c += 256)
    x[(int64_t)t * a.W + c] = Act<AT>::ld(e + c) * a.scale + Act<AT>::ld(b + c);
}

// bf16 tables, 8 channels per thread (W % 8 == 0)
__global__ __launch_bounds__(256) void hashed_embed_vec8_kernel(
    float* __restrict__ x, const int64_t* __restrict__ ids,
    const bf16* __restrict__ embed, const bf16* __restrict__ table, int* prev,
    const int* __restrict__ cu, const int* __restrict__ seq_lens,
    const int* __restrict__ slots, const int* __restrict__ token_seq,
    HashDims a, int single) {
  const int t = blockIdx.x;
  const int64_t row =
      hashed_row(t, ids, prev, cu, seq_lens, slots, token_seq, a, single);
  const bf16* e = embed + ids[t] * a.W;
  const bf16* b = table + row * a.W;
  for (int c = threadIdx.x * 8; c < a.W; c += 256 * 8) {
    const ushort8 u = *reinterpret_cast<const ushort8*>(e + c);
    const ushort8 v = *reinterpret_cast<const ushort8*>(b + c);
    float4v lo, hi;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      lo[i] = bf16_bits_to_float(u[i]) * a.scale + bf16_bits_to_float(v[i]);
      hi[i] = bf16_bits_to_float(u[4 + i]) * a.scale +
              bf16_bits_to_float(v[4 + i]);
    }
    float* xr = x + (int64_t)t * a.W + c;
    *reinterpret_cast<float4v*>(xr) = lo;
    *reinterpret_cast<float4v*>(xr + 4) = hi;
  }
}

// After the rows of a step with portions have read the old state.
__global__ __launch_bounds__(64) void prev_token_update_kernel(
    int* __restrict__ prev, const int64_t* __restrict__ ids,
    const int* __restrict__ cu, const int* __restrict__ slots, int S) {
  const int s = blockIdx.x * 64 + threadIdx.x;
  if (s >= S) return;
  if (cu[s + 1] > cu[s] && slots[s] >= 0) prev[slots[s]] = (int)ids[cu[s + 1] - 1];
}

// ------------------------------------------------- whole-row q/k norm, pages
struct RowNormDims {
  int64_t ldq, ldk, ldv;
  float eps, temp_coef;
  int temp_every, H, G, D, V, bs;
};

// One block per row, any sizes.
template <typename AT>
__global__ __launch_bounds__(256) void row_norm_qk_cache_kernel(
    AT* __restrict__ qo, const AT* __restrict__ q, const AT* __restrict__ k,
    const AT* __restrict__ v, const float* __restrict__ qw,
    const float* __restrict__ kw, const int64_t* __restrict__ positions,
    AT* __restrict__ k_cache, AT* __restrict__ v_cache,
    const int64_t* __restrict__ slot_mapping, RowNormDims a) {
  __shared__ float red[4], red2[4];
  const int64_t t = blockIdx.x;
  const int nq = a.H * a.D, nk = a.G * a.D, nv = a.G * a.V;
  const AT* qr = q + t * a.ldq;
  const AT* kr = k + t * a.ldk;
  const AT* vr = v + t * a.ldv;
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x; c < nq; c += 256) {
    const float z = Act<AT>::ld(qr + c);
    sq += z * z;
  }
  for (int c = threadIdx.x; c < nk; c += 256) {
    const float z = Act<AT>::ld(kr + c);
    sk += z * z;
  }
  sq = block_reduce_sum<256>(sq, red);
  sk = block_reduce_sum<256>(sk, red2);
  const float fq = query_factor(positions[t], a.temp_coef, a.temp_every) /
                   sqrtf(sq / (float)nq + a.eps);
  const float fk = 1.f / sqrtf(sk / (float)nk + a.eps);
  for (int c = threadIdx.x; c < nq; c += 256)
    Act<AT>::st(qo + t * nq + c, Act<AT>::ld(qr + c) * fq * qw[c]);
  const int64_t slot = slot_mapping[t];
  if (slot < 0) return;
  const int64_t page = slot / a.bs, at = slot % a.bs;
  for (int c = threadIdx.x; c < nk; c += 256)
    Act<AT>::st(k_cache + ((page * a.G + c / a.D) * a.bs + at) * a.D + c % a.D,
                Act<AT>::ld(kr + c) * fk * kw[c]);
  for (int c = threadIdx.x; c < nv; c += 256)
    Act<AT>::st(v_cache + ((page * a.G + c / a.V) * a.bs + at) * a.V + c % a.V,
                Act<AT>::ld(vr + c));
}

// bf16, 8 elements per access (head sizes and row strides multiples of 8),
// H * D <= 2048 * IT: the row stays in registers through the reduction.
template <int IT>
__global__ __launch_bounds__(256) void row_norm_qk_cache_vec8_kernel(
    bf16* __restrict__ qo, const bf16* __restrict__ q,
    const bf16* __restrict__ k, const bf16* __restrict__ v,
    const float* __restrict__ qw, const float* __restrict__ kw,
    const int64_t* __restrict__ positions, bf16* __restrict__ k_cache,
    bf16* __restrict__ v_cache, const int64_t* __restrict__ slot_mapping,
    RowNormDims a) {
  __shared__ float red[4], red2[4];
  const int64_t t = blockIdx.x;
  const int nq = a.H * a.D, nk = a.G * a.D, nv = a.G * a.V;
  ushort8 qv[IT], kv[IT];
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int c = (it * 256 + threadIdx.x) * 8;
    qv[it] = ushort8{};
    kv[it] = ushort8{};
    if (c < nq) qv[it] = *reinterpret_cast<const ushort8*>(q + t * a.ldq + c);
    if (c < nk) kv[it] = *reinterpret_cast<const ushort8*>(k + t * a.ldk + c);
  }
  const int64_t slot = slot_mapping[t];
  const int64_t page = slot / a.bs, at = slot % a.bs;
  if (slot >= 0) {
    for (int c = threadIdx.x * 8; c < nv; c += 256 * 8)
      *reinterpret_cast<ushort8*>(
          v_cache + ((page * a.G + c / a.V) * a.bs + at) * a.V + c % a.V) =
          *reinterpret_cast<const ushort8*>(v + t * a.ldv + c);
  }
#pragma unroll
  for (int it = 0; it < IT; ++it)
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float y = bf16_bits_to_float(qv[it][e]);
      const float z = bf16_bits_to_float(kv[it][e]);
      sq += y * y;
      sk += z * z;
    }
  sq = block_reduce_sum<256>(sq, red);
  sk = block_reduce_sum<256>(sk, red2);
  const float fq = query_factor(positions[t], a.temp_coef, a.temp_every) /
                   sqrtf(sq / (float)nq + a.eps);
  const float fk = 1.f / sqrtf(sk / (float)nk + a.eps);
  auto weighed = [](const ushort8& r, float f, const float* w) {
    const float4v lo = *reinterpret_cast<const float4v*>(w);
    const float4v hi = *reinterpret_cast<const float4v*>(w + 4);
    ushort8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e)
      o[e] = float_to_bf16_bits(bf16_bits_to_float(r[e]) * f *
                                (e < 4 ? lo[e] : hi[e - 4]));
    return o;
  };
#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int c = (it * 256 + threadIdx.x) * 8;
    if (c < nq)
      *reinterpret_cast<ushort8*>(qo + t * nq + c) = weighed(qv[it], fq, qw + c);
    if (c < nk && slot >= 0)
      *reinterpret_cast<ushort8*>(
          k_cache + ((page * a.G + c / a.D) * a.bs + at) * a.D + c % a.D) =
          weighed(kv[it], fk, kw + c);
  }
}

// ---------------------------------------------------------- squared relu
template <typename AT>
__global__ __launch_bounds__(256) void relu_square_kernel(
    AT* __restrict__ out, const AT* __restrict__ x, int64_t n) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const float z = fmaxf(Act<AT>::ld(x + i), 0.f);
  Act<AT>::st(out + i, z * z);
}

__global__ __launch_bounds__(256) void relu_square_vec8_kernel(
    bf16* __restrict__ out, const bf16* __restrict__ x, int64_t n8) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n8) return;
  const ushort8 v = *reinterpret_cast<const ushort8*>(x + i * 8);
  ushort8 o;
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const float z = fmaxf(bf16_bits_to_float(v[e]), 0.f);
    o[e] = float_to_bf16_bits(z * z);
  }
  *reinterpret_cast<ushort8*>(out + i * 8) = o;
}

}  // namespace arks

using namespace arks;

extern "C" void arks_seq_hashed_embed(
    void* x, const void* ids, const void* embed, const void* table, void* prev,
    const void* cu, const void* seq_lens, const void* slots,
    const void* token_seq, float scale, int64_t mul_prev, int64_t mul_cur,
    int64_t buckets, int T, int S, int W, int single, int act_f32,
    hipStream_t stream) {
  if (T == 0) return;
  const HashDims a{mul_prev, mul_cur, buckets, scale, W};
  if (!act_f32 && W % 8 == 0 &&
      (((uintptr_t)x | (uintptr_t)embed | (uintptr_t)table) & 15) == 0) {
    hipLaunchKernelGGL(hashed_embed_vec8_kernel, dim3(T), dim3(256), 0, stream,
                       (float*)x, (const int64_t*)ids, (const bf16*)embed,
                       (const bf16*)table, (int*)prev, (const int*)cu,
                       (const int*)seq_lens, (const int*)slots,
                       (const int*)token_seq, a, single);
  } else {
    SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
        (hashed_embed_kernel<AT>), dim3(T), dim3(256), 0, stream, (float*)x,
        (const int64_t*)ids, (const AT*)embed, (const AT*)table, (int*)prev,
        (const int*)cu, (const int*)seq_lens, (const int*)slots,
        (const int*)token_seq, a, single));
  }
  if (!single)
    hipLaunchKernelGGL(prev_token_update_kernel, dim3((S + 63) / 64), dim3(64),
                       0, stream, (int*)prev, (const int64_t*)ids,
                       (const int*)cu, (const int*)slots, S);
}

extern "C" void arks_seq_row_norm_qk_cache(
    void* qo, const void* q, const void* k, const void* v, int64_t ldq,
    int64_t ldk, int64_t ldv, const void* qw, const void* kw, float eps,
    const void* positions, float temp_coef, int temp_every, void* k_cache,
    void* v_cache, const void* slot_mapping, int T, int H, int G, int D, int V,
    int bs, int act_f32, hipStream_t stream) {
  if (T == 0) return;
  const RowNormDims a{ldq, ldk, ldv, eps, temp_coef, temp_every,
                      H,   G,   D,   V,   bs};
  if (!act_f32 && D % 8 == 0 && V % 8 == 0 && ldq % 8 == 0 && ldk % 8 == 0 &&
      ldv % 8 == 0 && H * D <= 8192 &&
      (((uintptr_t)qo | (uintptr_t)q | (uintptr_t)k | (uintptr_t)v |
        (uintptr_t)qw | (uintptr_t)kw | (uintptr_t)k_cache |
        (uintptr_t)v_cache) & 15) == 0) {
#define RN(IT)                                                                \
  hipLaunchKernelGGL((row_norm_qk_cache_vec8_kernel<IT>), dim3(T), dim3(256), \
                     0, stream, (bf16*)qo, (const bf16*)q, (const bf16*)k,    \
                     (const bf16*)v, (const float*)qw, (const float*)kw,      \
                     (const int64_t*)positions, (bf16*)k_cache,               \
                     (bf16*)v_cache, (const int64_t*)slot_mapping, a)
    if (H * D <= 2048) RN(1);
    else if (H * D <= 4096) RN(2);
    else RN(4);
#undef RN
    return;
  }
  SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
      (row_norm_qk_cache_kernel<AT>), dim3(T), dim3(256), 0, stream, (AT*)qo,
      (const AT*)q, (const AT*)k, (const AT*)v, (const float*)qw,
      (const float*)kw, (const int64_t*)positions, (AT*)k_cache, (AT*)v_cache,
      (const int64_t*)slot_mapping, a));
}

extern "C" void arks_seq_relu_square(void* out, const void* x, int64_t n,
                                     int act_f32, hipStream_t stream) {
  if (n == 0) return;
  if (!act_f32 && n % 8 == 0 && (((uintptr_t)out | (uintptr_t)x) & 15) == 0) {
    hipLaunchKernelGGL(relu_square_vec8_kernel,
                       dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0,
                       stream, (bf16*)out, (const bf16*)x, n / 8);
    return;
  }
  SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
      (relu_square_kernel<AT>), dim3((unsigned)((n + 255) / 256)), dim3(256),
      0, stream, (AT*)out, (const AT*)x, n));
}
