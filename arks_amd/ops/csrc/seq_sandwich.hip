// Row kernels of the sandwich-norm blocks (arks_amd/models/hybrid.py
// SandwichBlock), bf16 or float rows, fp32 arithmetic:
//
//   residual_sandwich_norm  x += mult * (rms_norm(y) * w_post + rms_norm(y2)
//       * w_post2) on the fp32 residual (y and y2, the previous sublayer's
//       results, optional; without a weight a result is added as it is), then
//       h = rms_norm(x) * w_pre (optional), the next sublayer's input
//   head_gate  out[t, h] = o[t, h] * sigmoid(gate[t, h]) * out_scale
//   softcap    x = cap * tanh(x / cap) in place
#include "seq_common.h"

namespace arks {

// One block per row, any width.
template <typename AT>
__global__ __launch_bounds__(256) void residual_sandwich_norm_kernel(
    float* __restrict__ x, AT* __restrict__ h, const AT* __restrict__ y,
    const float* __restrict__ w_post, const AT* __restrict__ y2,
    const float* __restrict__ w_post2, float mult,
    const float* __restrict__ w_pre, float eps, int C) {
  __shared__ float red[4], red2[4], red3[4];
  const int64_t t = blockIdx.x;
  float* xr = x + t * C;
  auto row_scale = [&](const AT* r, float* scratch) {
    float ss = 0.f;
    for (int c = threadIdx.x; c < C; c += 256) {
      const float v = Act<AT>::ld(r + t * C + c);
      ss += v * v;
    }
    ss = block_reduce_sum<256>(ss, scratch);
    return 1.f / sqrtf(ss / (float)C + eps);
  };
  const float ry = y && w_post ? row_scale(y, red) : 1.f;
  const float ry2 = y2 && w_post2 ? row_scale(y2, red3) : 1.f;
  float ss = 0.f;
  for (int c = threadIdx.x; c < C; c += 256) {
    float v = xr[c];
    if (y) {
      float z = Act<AT>::ld(y + t * C + c);
      if (w_post) z *= ry * w_post[c];
      if (y2) {
        const float z2 = Act<AT>::ld(y2 + t * C + c);
        z += w_post2 ? z2 * ry2 * w_post2[c] : z2;
      }
      v += mult * z;
      xr[c] = v;
    }
    ss += v * v;
  }
  if (!h) return;
  ss = block_reduce_sum<256>(ss, red2);
  const float rx = 1.f / sqrtf(ss / (float)C + eps);
  for (int c = threadIdx.x; c < C; c += 256)
    Act<AT>::st(h + t * C + c, xr[c] * rx * w_pre[c]);  // own writes of x
}

// bf16 rows, C % 8 == 0, C <= 2048 * IT: every thread keeps its pieces of
// the rows in registers through the reductions. TWO: y2 is given.
template <int IT, bool TWO>
__global__ __launch_bounds__(256) void residual_sandwich_norm_vec8_kernel(
    float* __restrict__ x, bf16* __restrict__ h, const bf16* __restrict__ y,
    const float* __restrict__ w_post, const bf16* __restrict__ y2,
    const float* __restrict__ w_post2, float mult,
    const float* __restrict__ w_pre, float eps, int C) {
  __shared__ float red[4], red2[4], red3[4];
  const int64_t t = blockIdx.x;
  float* xr = x + t * C;
  float v[IT][8];
#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int c = (it * 256 + threadIdx.x) * 8;
    if (c < C) {
      const float4v a = *reinterpret_cast<const float4v*>(xr + c);
      const float4v b = *reinterpret_cast<const float4v*>(xr + c + 4);
#pragma unroll
      for (int e = 0; e < 4; ++e) { v[it][e] = a[e]; v[it][4 + e] = b[e]; }
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e) v[it][e] = 0.f;
    }
  }
  if (y) {
    ushort8 yv[IT], zv[IT];
    float ss = 0.f, ss2 = 0.f;
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int c = (it * 256 + threadIdx.x) * 8;
      yv[it] = ushort8{};
      zv[it] = ushort8{};
      if (c < C) {
        yv[it] = *reinterpret_cast<const ushort8*>(y + t * C + c);
        if (TWO) zv[it] = *reinterpret_cast<const ushort8*>(y2 + t * C + c);
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float a = bf16_bits_to_float(yv[it][e]);
        const float b = bf16_bits_to_float(zv[it][e]);
        ss += a * a;
        if (TWO) ss2 += b * b;
      }
    }
    float ry = mult, ry2 = mult;
    if (w_post) ry /= sqrtf(block_reduce_sum<256>(ss, red) / (float)C + eps);
    if (TWO && w_post2)
      ry2 /= sqrtf(block_reduce_sum<256>(ss2, red3) / (float)C + eps);
    auto add_row = [&](int it, int c, const ushort8& r, const float* w,
                       float f) {
      float4v wa = {1.f, 1.f, 1.f, 1.f}, wb = {1.f, 1.f, 1.f, 1.f};
      if (w) {
        wa = *reinterpret_cast<const float4v*>(w + c);
        wb = *reinterpret_cast<const float4v*>(w + c + 4);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        v[it][e] += bf16_bits_to_float(r[e]) * f * wa[e];
        v[it][4 + e] += bf16_bits_to_float(r[4 + e]) * f * wb[e];
      }
    };
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int c = (it * 256 + threadIdx.x) * 8;
      if (c < C) {
        add_row(it, c, yv[it], w_post, ry);
        if (TWO) add_row(it, c, zv[it], w_post2, ry2);
        float4v a, b;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          a[e] = v[it][e];
          b[e] = v[it][4 + e];
        }
        *reinterpret_cast<float4v*>(xr + c) = a;
        *reinterpret_cast<float4v*>(xr + c + 4) = b;
      }
    }
  }
  if (!h) return;
  float ss = 0.f;
#pragma unroll
  for (int it = 0; it < IT; ++it)
#pragma unroll
    for (int e = 0; e < 8; ++e) ss += v[it][e] * v[it][e];
  ss = block_reduce_sum<256>(ss, red2);
  const float rx = 1.f / sqrtf(ss / (float)C + eps);
#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int c = (it * 256 + threadIdx.x) * 8;
    if (c < C) {
      const float4v wa = *reinterpret_cast<const float4v*>(w_pre + c);
      const float4v wb = *reinterpret_cast<const float4v*>(w_pre + c + 4);
      ushort8 o;
#pragma unroll
      for (int e = 0; e < 8; ++e)
        o[e] = float_to_bf16_bits(v[it][e] * rx * (e < 4 ? wa[e] : wb[e - 4]));
      *reinterpret_cast<ushort8*>(h + t * C + c) = o;
    }
  }
}

// One thread per element; o and out [T, H, V] with strides (lit, lih) and
// (lot, loh), dense last dim; may be the same view.
template <typename AT>
__global__ __launch_bounds__(256) void head_gate_kernel(
    AT* out, int64_t lot, int64_t loh, const AT* o, int64_t lit, int64_t lih,
    const AT* __restrict__ gate, int64_t ldg, float out_scale, int64_t n,
    int H, int V) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const int v = (int)(i % V);
  const int hh = (int)((i / V) % H);
  const int64_t t = i / ((int64_t)V * H);
  const float f =
      gate ? sigmoid_f(Act<AT>::ld(gate + t * ldg + hh)) * out_scale : out_scale;
  Act<AT>::st(out + t * lot + hh * loh + v,
              Act<AT>::ld(o + t * lit + hh * lih + v) * f);
}

// bf16, 8 elements per thread (V and all strides multiples of 8)
__global__ __launch_bounds__(256) void head_gate_vec8_kernel(
    bf16* out, int64_t lot, int64_t loh, const bf16* o, int64_t lit,
    int64_t lih, const bf16* __restrict__ gate, int64_t ldg, float out_scale,
    int64_t n8, int H, int V) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n8) return;
  const int V8 = V / 8;
  const int v = (int)(i % V8) * 8;
  const int hh = (int)((i / V8) % H);
  const int64_t t = i / ((int64_t)V8 * H);
  const float f = gate ? out_scale /
                             (1.f + __expf(-bf16_bits_to_float(gate[t * ldg + hh])))
                       : out_scale;
  const ushort8 u =
      *reinterpret_cast<const ushort8*>(o + t * lit + hh * lih + v);
  ushort8 r;
#pragma unroll
  for (int e = 0; e < 8; ++e)
    r[e] = float_to_bf16_bits(bf16_bits_to_float(u[e]) * f);
  *reinterpret_cast<ushort8*>(out + t * lot + hh * loh + v) = r;
}

__global__ __launch_bounds__(256) void softcap_kernel(float* __restrict__ x,
                                                      int64_t n, float cap) {
  const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (i + 4 <= n) {
    float4v v = *reinterpret_cast<const float4v*>(x + i);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = cap * tanhf(v[e] / cap);
    *reinterpret_cast<float4v*>(x + i) = v;
  } else {
    for (int64_t j = i; j < n; ++j) x[j] = cap * tanhf(x[j] / cap);
  }
}

}  // namespace arks

using namespace arks;

extern "C" void arks_seq_residual_sandwich_norm(
    void* x, void* h, const void* y, const void* w_post, const void* y2,
    const void* w_post2, float mult, const void* w_pre, float eps, int64_t T,
    int C, int act_f32, hipStream_t stream) {
  if (T == 0) return;
  const bool aligned = (((uintptr_t)x | (uintptr_t)h | (uintptr_t)y |
                         (uintptr_t)w_post | (uintptr_t)y2 |
                         (uintptr_t)w_post2 | (uintptr_t)w_pre) & 15) == 0;
  if (!act_f32 && C % 8 == 0 && C <= 8192 && aligned) {
#define SN(IT, TWO)                                                           \
  hipLaunchKernelGGL((residual_sandwich_norm_vec8_kernel<IT, TWO>), dim3(T),  \
                     dim3(256), 0, stream, (float*)x, (bf16*)h,               \
                     (const bf16*)y, (const float*)w_post, (const bf16*)y2,   \
                     (const float*)w_post2, mult, (const float*)w_pre, eps, C)
#define SN2(IT)        \
  do {                 \
    if (y2) SN(IT, true); \
    else SN(IT, false);   \
  } while (0)
    if (C <= 2048) SN2(1);
    else if (C <= 4096) SN2(2);
    else SN2(4);
#undef SN2
#undef SN
    return;
  }
  SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
      (residual_sandwich_norm_kernel<AT>), dim3(T), dim3(256), 0, stream,
      (float*)x, (AT*)h, (const AT*)y, (const float*)w_post, (const AT*)y2,
      (const float*)w_post2, mult, (const float*)w_pre, eps, C));
}

extern "C" void arks_seq_softcap(void* x, int64_t n, float cap,
                                 hipStream_t stream) {
  if (n == 0) return;
  hipLaunchKernelGGL(softcap_kernel, dim3((unsigned)((n + 1023) / 1024)),
                     dim3(256), 0, stream, (float*)x, n, cap);
}

extern "C" void arks_seq_head_gate(void* out, int64_t lot, int64_t loh,
                                   const void* o, int64_t lit, int64_t lih,
                                   const void* gate, int64_t ldg,
                                   float out_scale, int64_t T, int H, int V,
                                   int act_f32, hipStream_t stream) {
  const int64_t n = T * H * (int64_t)V;
  if (n == 0) return;
  if (!act_f32 && V % 8 == 0 && lot % 8 == 0 && loh % 8 == 0 && lit % 8 == 0 &&
      lih % 8 == 0 && (((uintptr_t)out | (uintptr_t)o) & 15) == 0) {
    hipLaunchKernelGGL(head_gate_vec8_kernel,
                       dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0,
                       stream, (bf16*)out, lot, loh, (const bf16*)o, lit, lih,
                       (const bf16*)gate, ldg, out_scale, n / 8, H, V);
    return;
  }
  SEQ_DISPATCH_ACT(act_f32, hipLaunchKernelGGL(
      (head_gate_kernel<AT>), dim3((unsigned)((n + 255) / 256)), dim3(256), 0,
      stream, (AT*)out, lot, loh, (const AT*)o, lit, lih, (const AT*)gate, ldg,
      out_scale, n, H, V));
}
