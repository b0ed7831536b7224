// Row kernels of the shared-norm blocks and of latent attention:
//   residual_tanh_norm: x (fp32 residual) += mult * y, then
//       h = tanh(alpha x) * w + b  — a norm without statistics, so nothing
//       is reduced over the row and the kernel is purely elementwise;
//   latent_prepare: RMS norm of the query latent; RMS norm of the key/value
//       latent and rotation of the shared key part, written to the row's
//       place in the paged latent cache;
//   latent_query: [absorbed query | rotated part] per head;
//   latent_pages: per-head key and value pages from up-projected rows and
//       the shared key part.
#include "seq_common.h"

namespace arks {

// tanh for rows that are rounded to bf16 afterwards: 1 - 2 / (e^{2z} + 1)
// with the hardware exponential; absolute error ~1e-7.
template <typename AT>
__device__ __forceinline__ float tanh_act(float z);
template <>
__device__ __forceinline__ float tanh_act<float>(float z) { return tanhf(z); }
template <>
__device__ __forceinline__ float tanh_act<bf16>(float z) {
  const float e = __expf(2.f * fminf(fmaxf(z, -15.f), 15.f));
  return 1.f - 2.f / (e + 1.f);
}

// One thread per element. y, h: [T, C] dense; xa: [T, C] with row stride.
template <typename AT>
__global__ __launch_bounds__(256) void residual_tanh_norm_kernel(
    float* __restrict__ x, AT* __restrict__ h, AT* __restrict__ xa,
    int64_t ldxa, const AT* __restrict__ y, float mult,
    const float* __restrict__ alpha, const float* __restrict__ w,
    const float* __restrict__ b, int64_t n, int C) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  float v = x[i];
  if (y) {
    v += mult * Act<AT>::ld(y + i);
    x[i] = v;
  }
  const int64_t t = i / C;
  const int c = (int)(i - t * C);
  if (xa) Act<AT>::st(xa + t * ldxa + c, v);
  if (h) Act<AT>::st(h + i, tanh_act<AT>(alpha[0] * v) * w[c] + b[c]);
}

// bf16 rows, 8 elements per thread (C % 8 == 0, 16-byte aligned rows).
__global__ __launch_bounds__(256) void residual_tanh_norm_vec8_kernel(
    float* __restrict__ x, bf16* __restrict__ h, bf16* __restrict__ xa,
    int64_t ldxa, const bf16* __restrict__ y, float mult,
    const float* __restrict__ alpha, const float* __restrict__ w,
    const float* __restrict__ b, int64_t n, int C) {
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 8;
  if (i >= n) return;
  float v[8];
  {
    const float4v a0 = *reinterpret_cast<const float4v*>(x + i);
    const float4v a1 = *reinterpret_cast<const float4v*>(x + i + 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) { v[e] = a0[e]; v[4 + e] = a1[e]; }
  }
  if (y) {
    const ushort8 yv = *reinterpret_cast<const ushort8*>(y + i);
    float4v o0, o1;
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] += mult * bf16_bits_to_float(yv[e]);
#pragma unroll
    for (int e = 0; e < 4; ++e) { o0[e] = v[e]; o1[e] = v[4 + e]; }
    *reinterpret_cast<float4v*>(x + i) = o0;
    *reinterpret_cast<float4v*>(x + i + 4) = o1;
  }
  const int64_t t = i / C;
  const int c = (int)(i - t * C);
  if (xa) {
    ushort8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = float_to_bf16_bits(v[e]);
    *reinterpret_cast<ushort8*>(xa + t * ldxa + c) = o;
  }
  if (h) {
    const float al = alpha[0];
    const float4v w0 = *reinterpret_cast<const float4v*>(w + c);
    const float4v w1 = *reinterpret_cast<const float4v*>(w + c + 4);
    const float4v b0 = *reinterpret_cast<const float4v*>(b + c);
    const float4v b1 = *reinterpret_cast<const float4v*>(b + c + 4);
    ushort8 o;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      o[e] = float_to_bf16_bits(tanh_act<bf16>(al * v[e]) * w0[e] + b0[e]);
      o[4 + e] =
          float_to_bf16_bits(tanh_act<bf16>(al * v[4 + e]) * w1[e] + b1[e]);
    }
    *reinterpret_cast<ushort8*>(h + i) = o;
  }
}

// Pair i of a rotated part of 2P dims: (2i, 2i + 1), or (i, i + P) half-split;
// cos and sin times mag.
template <typename AT>
__device__ __forceinline__ void turn_pair(AT* dst, const AT* src, int i, int P,
                                          float angle, int half_split,
                                          float mag) {
  float sn, cs;
  sincosf(angle, &sn, &cs);
  sn *= mag;
  cs *= mag;
  const int i0 = half_split ? i : 2 * i, i1 = half_split ? i + P : 2 * i + 1;
  const float a = Act<AT>::ld(src + i0), b = Act<AT>::ld(src + i1);
  Act<AT>::st(dst + i0, a * cs - b * sn);
  Act<AT>::st(dst + i1, b * cs + a * sn);
}

// One block per row. cq [T, Rq] (row stride ldq) -> cqn [T, Rq] dense;
// ckv [T, Rk + 2P] (row stride ldk) -> its cache row.
template <typename AT>
__global__ __launch_bounds__(256) void latent_prepare_kernel(
    AT* __restrict__ cqn, const AT* __restrict__ cq, int64_t ldq,
    const AT* __restrict__ ckv, int64_t ldk, const float* __restrict__ qw,
    const float* __restrict__ kw, float eps,
    const int64_t* __restrict__ positions, const float* __restrict__ freq,
    AT* __restrict__ cache, const int64_t* __restrict__ slot_mapping, int Rq,
    int Rk, int P, int half_split, float mag) {
  __shared__ float scratch[4];
  __shared__ float scratch2[4];
  const int t = blockIdx.x;
  const AT* qr = cq + (int64_t)t * ldq;
  float ss = 0.f;
  for (int i = threadIdx.x; i < Rq; i += 256) {
    const float a = Act<AT>::ld(qr + i);
    ss += a * a;
  }
  ss = block_reduce_sum<256>(ss, scratch);
  const float rq = 1.f / sqrtf(ss / (float)Rq + eps);
  for (int i = threadIdx.x; i < Rq; i += 256)
    Act<AT>::st(cqn + (int64_t)t * Rq + i, Act<AT>::ld(qr + i) * rq * qw[i]);
  const int64_t slot = slot_mapping[t];
  if (slot < 0) return;  // uniform over the block
  const AT* kr = ckv + (int64_t)t * ldk;
  AT* dst = cache + slot * (int64_t)(Rk + 2 * P);
  float s2 = 0.f;
  for (int i = threadIdx.x; i < Rk; i += 256) {
    const float a = Act<AT>::ld(kr + i);
    s2 += a * a;
  }
  s2 = block_reduce_sum<256>(s2, scratch2);
  const float rk = 1.f / sqrtf(s2 / (float)Rk + eps);
  for (int i = threadIdx.x; i < Rk; i += 256)
    Act<AT>::st(dst + i, Act<AT>::ld(kr + i) * rk * kw[i]);
  const float pos = (float)positions[t];
  for (int i = threadIdx.x; i < P; i += 256)
    turn_pair<AT>(dst + Rk, kr + Rk, i, P, pos * freq[i], half_split, mag);
}

// bf16 rows, 16-byte accesses (Rq, Rk, strides multiples of 8, half-split
// pairs with P a multiple of 8, Rq + Rk <= 8 * 256 * LP_IT): the row's pieces
// stay in registers between the sums of squares and the scaling.
constexpr int LP_IT = 2;

__global__ __launch_bounds__(256) void latent_prepare_vec8_kernel(
    bf16* __restrict__ cqn, const bf16* __restrict__ cq, int64_t ldq,
    const bf16* __restrict__ ckv, int64_t ldk, const float* __restrict__ qw,
    const float* __restrict__ kw, float eps,
    const int64_t* __restrict__ positions, const float* __restrict__ freq,
    bf16* __restrict__ cache, const int64_t* __restrict__ slot_mapping, int Rq,
    int Rk, int P, float mag) {
  __shared__ float red[4][2];
  const int t = blockIdx.x;
  const int nq = Rq / 8, n = nq + Rk / 8;
  const int64_t slot = slot_mapping[t];
  bf16* dst = cache + (slot < 0 ? 0 : slot) * (int64_t)(Rk + 2 * P);
  const bf16* kr = ckv + (int64_t)t * ldk;
  ushort8 in[LP_IT];
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int it = 0; it < LP_IT; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n) {
      in[it] = *reinterpret_cast<const ushort8*>(
          i < nq ? cq + (int64_t)t * ldq + i * 8 : kr + (i - nq) * 8);
      float s = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float a = bf16_bits_to_float(in[it][e]);
        s += a * a;
      }
      (i < nq ? sq : sk) += s;
    }
  }
  // the rotated part: the last threads, 8 pairs each
  const int rot = 255 - (int)threadIdx.x;
  if (rot < P / 8 && slot >= 0) {
    const float pos = (float)positions[t];
    const ushort8 a = *reinterpret_cast<const ushort8*>(kr + Rk + rot * 8);
    const ushort8 b = *reinterpret_cast<const ushort8*>(kr + Rk + P + rot * 8);
    ushort8 x, y;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      float sn, cs;
      sincosf(pos * freq[rot * 8 + e], &sn, &cs);
      const float u = bf16_bits_to_float(a[e]), v = bf16_bits_to_float(b[e]);
      x[e] = float_to_bf16_bits((u * cs - v * sn) * mag);
      y[e] = float_to_bf16_bits((v * cs + u * sn) * mag);
    }
    *reinterpret_cast<ushort8*>(dst + Rk + rot * 8) = x;
    *reinterpret_cast<ushort8*>(dst + Rk + P + rot * 8) = y;
  }
  sq = wave_reduce_sum(sq);
  sk = wave_reduce_sum(sk);
  if (threadIdx.x % 64 == 0) {
    red[threadIdx.x / 64][0] = sq;
    red[threadIdx.x / 64][1] = sk;
  }
  __syncthreads();
  sq = red[0][0] + red[1][0] + red[2][0] + red[3][0];
  sk = red[0][1] + red[1][1] + red[2][1] + red[3][1];
  const float rq = 1.f / sqrtf(sq / (float)Rq + eps);
  const float rk = 1.f / sqrtf(sk / (float)Rk + eps);
#pragma unroll
  for (int it = 0; it < LP_IT; ++it) {
    const int i = it * 256 + threadIdx.x;
    if (i < n) {
      const bool is_q = i < nq;
      const float* w = is_q ? qw + i * 8 : kw + (i - nq) * 8;
      const float r = is_q ? rq : rk;
      ushort8 o;
#pragma unroll
      for (int e = 0; e < 8; ++e)
        o[e] = float_to_bf16_bits(bf16_bits_to_float(in[it][e]) * r * w[e]);
      if (is_q)
        *reinterpret_cast<ushort8*>(cqn + (int64_t)t * Rq + i * 8) = o;
      else if (slot >= 0)
        *reinterpret_cast<ushort8*>(dst + (i - nq) * 8) = o;
    }
  }
}

// out [T, H, Rk + 2P] = [q_abs[h, t, :] | rotated q[t, h, D:]]; one block
// per row, waves over heads. q_abs null: the first part is q[t, h, :D], and
// out may be q itself.
template <typename AT>
__global__ __launch_bounds__(256) void latent_query_kernel(
    AT* out, const AT* q, const AT* __restrict__ q_abs,
    const int64_t* __restrict__ positions, const float* __restrict__ freq,
    int T, int H, int D, int Rk, int P, int half_split, float mag) {
  const int t = blockIdx.x;
  const int wave = threadIdx.x / 64, lane = threadIdx.x % 64;
  const float pos = (float)positions[t];
  for (int hh = wave; hh < H; hh += 4) {
    AT* dst = out + ((int64_t)t * H + hh) * (Rk + 2 * P);
    // without q_abs the plain part is q's own (Rk == D)
    const AT* src = q_abs ? q_abs + ((int64_t)hh * T + t) * Rk
                          : q + ((int64_t)t * H + hh) * (D + 2 * P);
    if (dst != src)
      for (int i = lane; i < Rk; i += 64) dst[i] = src[i];
    const AT* qr = q + ((int64_t)t * H + hh) * (D + 2 * P) + D;
    for (int i = lane; i < P; i += 64)
      turn_pair<AT>(dst + Rk, qr, i, P, pos * freq[i], half_split, mag);
  }
}

// bf16, 16-byte accesses (D, Rk multiples of 8, half-split pairs with P a
// multiple of 8): the row's sines and cosines are evaluated once into LDS.
constexpr int LQ_MAX_P = 128;

__global__ __launch_bounds__(256) void latent_query_vec8_kernel(
    bf16* out, const bf16* q, const bf16* __restrict__ q_abs,
    const int64_t* __restrict__ positions, const float* __restrict__ freq,
    int T, int H, int D, int Rk, int P, float mag) {
  __shared__ float sn_s[LQ_MAX_P], cs_s[LQ_MAX_P];
  const int64_t t = blockIdx.x;
  const float pos = (float)positions[t];
  for (int i = threadIdx.x; i < P; i += 256) {
    float sn, cs;
    sincosf(pos * freq[i], &sn, &cs);
    sn_s[i] = sn * mag;
    cs_s[i] = cs * mag;
  }
  __syncthreads();
  // without q_abs the plain part is q's own (Rk == D), already there if out
  // is q
  const int np = !q_abs && out == q ? 0 : Rk / 8;
  const int per = np + P / 8;  // pieces of a head: plain ones, pairs
  for (int i = threadIdx.x; i < H * per; i += 256) {
    const int hh = i / per, j = i % per;
    const bf16* qr = q + (t * H + hh) * (D + 2 * P);
    bf16* dst = out + (t * H + hh) * (Rk + 2 * P);
    if (j < np) {
      const bf16* src = q_abs ? q_abs + ((int64_t)hh * T + t) * Rk : qr;
      *reinterpret_cast<ushort8*>(dst + j * 8) =
          *reinterpret_cast<const ushort8*>(src + j * 8);
      continue;
    }
    const int p0 = (j - np) * 8;
    const ushort8 a = *reinterpret_cast<const ushort8*>(qr + D + p0);
    const ushort8 b = *reinterpret_cast<const ushort8*>(qr + D + P + p0);
    ushort8 x, y;
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float u = bf16_bits_to_float(a[e]), v = bf16_bits_to_float(b[e]);
      const float sn = sn_s[p0 + e], cs = cs_s[p0 + e];
      x[e] = float_to_bf16_bits(u * cs - v * sn);
      y[e] = float_to_bf16_bits(v * cs + u * sn);
    }
    *reinterpret_cast<ushort8*>(dst + Rk + p0) = x;
    *reinterpret_cast<ushort8*>(dst + Rk + P + p0) = y;
  }
}

// One block per (page, head). All sizes and row strides count pieces PT.
template <typename PT>
__global__ __launch_bounds__(256) void latent_pages_kernel(
    PT* __restrict__ kt, PT* __restrict__ vt, const PT* __restrict__ k_up,
    const PT* __restrict__ v_up, const PT* __restrict__ lat, int64_t ld_lat,
    int bs, int H, int D, int R, int V, int rank) {
  const int64_t page = blockIdx.x, head = blockIdx.y;
  const int64_t row0 = page * bs, to = (page * H + head) * bs;
  const int DR = D + R, nk = bs * DR, n = nk + bs * V;
  for (int i = threadIdx.x; i < n; i += 256) {
    if (i < nk) {
      const int t = i / DR, c = i % DR;
      const int64_t row = row0 + t;
      kt[(to + t) * DR + c] = c < D ? k_up[(row * H + head) * D + c]
                                    : lat[row * ld_lat + rank + c - D];
    } else {
      const int t = (i - nk) / V, c = (i - nk) % V;
      vt[(to + t) * V + c] = v_up[((row0 + t) * H + head) * V + c];
    }
  }
}

}  // namespace arks

using namespace arks;

extern "C" void arks_seq_residual_tanh_norm(
    void* x, void* h, void* xa, int64_t ldxa, const void* y, float mult,
    const void* alpha, const void* w, const void* b, int64_t T, int C,
    int act_f32, hipStream_t stream) {
  const int64_t n = T * C;
  if (n == 0) return;
  const bool aligned = (((uintptr_t)x | (uintptr_t)h | (uintptr_t)xa |
                         (uintptr_t)y | (uintptr_t)w | (uintptr_t)b) & 15) == 0;
  if (!act_f32 && C % 8 == 0 && ldxa % 8 == 0 && aligned) {
    hipLaunchKernelGGL(residual_tanh_norm_vec8_kernel,
                       dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0,
                       stream, (float*)x, (bf16*)h, (bf16*)xa, ldxa,
                       (const bf16*)y, mult, (const float*)alpha,
                       (const float*)w, (const float*)b, n, C);
    return;
  }
  SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
      (residual_tanh_norm_kernel<AT>), dim3((unsigned)((n + 255) / 256)),
      dim3(256), 0, stream, (float*)x, (AT*)h, (AT*)xa, ldxa, (const AT*)y,
      mult, (const float*)alpha, (const float*)w, (const float*)b, n, C));
}

extern "C" void arks_seq_latent_prepare(
    void* cqn, const void* cq, int64_t ldq, const void* ckv, int64_t ldk,
    const void* qw, const void* kw, float eps, const void* positions,
    const void* freq, void* cache, const void* slot_mapping, int T, int Rq,
    int Rk, int P, int half_split, float mag, int act_f32,
    hipStream_t stream) {
  if (T == 0) return;
  if (!act_f32 && half_split && Rq % 8 == 0 && Rk % 8 == 0 && P % 8 == 0 &&
      P <= 1024 && Rq + Rk <= 8 * 256 * LP_IT && ldq % 8 == 0 && ldk % 8 == 0 &&
      (((uintptr_t)cqn | (uintptr_t)cq | (uintptr_t)ckv | (uintptr_t)cache) &
       15) == 0) {
    hipLaunchKernelGGL(latent_prepare_vec8_kernel, dim3(T), dim3(256), 0,
                       stream, (bf16*)cqn, (const bf16*)cq, ldq,
                       (const bf16*)ckv, ldk, (const float*)qw,
                       (const float*)kw, eps, (const int64_t*)positions,
                       (const float*)freq, (bf16*)cache,
                       (const int64_t*)slot_mapping, Rq, Rk, P, mag);
    return;
  }
  SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
      (latent_prepare_kernel<AT>), dim3(T), dim3(256), 0, stream, (AT*)cqn,
      (const AT*)cq, ldq, (const AT*)ckv, ldk, (const float*)qw,
      (const float*)kw, eps, (const int64_t*)positions, (const float*)freq,
      (AT*)cache, (const int64_t*)slot_mapping, Rq, Rk, P, half_split, mag));
}

extern "C" void arks_seq_latent_query(void* out, const void* q,
                                      const void* q_abs, const void* positions,
                                      const void* freq, int T, int H, int D,
                                      int Rk, int P, int half_split, float mag,
                                      int act_f32, hipStream_t stream) {
  if (T == 0) return;
  if (!act_f32 && half_split && D % 8 == 0 && Rk % 8 == 0 && P % 8 == 0 &&
      P <= LQ_MAX_P &&
      (((uintptr_t)out | (uintptr_t)q | (uintptr_t)q_abs) & 15) == 0) {
    hipLaunchKernelGGL(latent_query_vec8_kernel, dim3(T), dim3(256), 0, stream,
                       (bf16*)out, (const bf16*)q, (const bf16*)q_abs,
                       (const int64_t*)positions, (const float*)freq, T, H, D,
                       Rk, P, mag);
    return;
  }
  SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
      (latent_query_kernel<AT>), dim3(T), dim3(256), 0, stream, (AT*)out,
      (const AT*)q, (const AT*)q_abs, (const int64_t*)positions,
      (const float*)freq, T, H, D, Rk, P, half_split, mag));
}

extern "C" void arks_seq_latent_pages(void* kt, void* vt, const void* k_up,
                                      const void* v_up, const void* lat,
                                      int64_t ld_lat, int NB, int bs, int H,
                                      int D, int R, int V, int rank,
                                      int elem_bytes, hipStream_t stream) {
  if (NB == 0) return;
  const int per = 16 / elem_bytes;  // elements of a 16-byte piece
  const dim3 grid(NB, H);
  if (D % per == 0 && R % per == 0 && V % per == 0 && rank % per == 0 &&
      ld_lat % per == 0 &&
      (((uintptr_t)kt | (uintptr_t)vt | (uintptr_t)k_up | (uintptr_t)v_up |
        (uintptr_t)lat) & 15) == 0) {
    hipLaunchKernelGGL((latent_pages_kernel<uint4>), grid, dim3(256), 0, stream,
                       (uint4*)kt, (uint4*)vt, (const uint4*)k_up,
                       (const uint4*)v_up, (const uint4*)lat, ld_lat / per, bs,
                       H, D / per, R / per, V / per, rank / per);
  } else if (elem_bytes == 4) {
    hipLaunchKernelGGL((latent_pages_kernel<uint32_t>), grid, dim3(256), 0,
                       stream, (uint32_t*)kt, (uint32_t*)vt,
                       (const uint32_t*)k_up, (const uint32_t*)v_up,
                       (const uint32_t*)lat, ld_lat, bs, H, D, R, V, rank);
  } else {
    hipLaunchKernelGGL((latent_pages_kernel<uint16_t>), grid, dim3(256), 0,
                       stream, (uint16_t*)kt, (uint16_t*)vt,
                       (const uint16_t*)k_up, (const uint16_t*)v_up,
                       (const uint16_t*)lat, ld_lat, bs, H, D, R, V, rank);
  }
}
