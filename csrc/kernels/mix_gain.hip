// Row kernels of layers whose norms are single gains (a norm before and after every sublayer),
// and of feed-forwards with a polynomial norm unit.
//
//   gain_sandwich    Y = y [+ sigmoid(s) y2] [+ w h_in];  x += g_post Y / rms(Y);
//                    out = g_pre x / rms(x)              (fp32 stream x; each part optional)
//                    y2 with one logit s per row is a gated shared expert, h_in with one weight
//                    per row the share of the experts that hand their input on unchanged
//   poly_norm_rows   a N(z) + b N(z^2) + c N(z^3) + e,  N(u) = u / sqrt(mean(u^2) + eps)
//
// One workgroup per row.  Sums, norms and the stream are fp32 whatever the activation type.
#include "mix_common.h"

namespace rfqmix {

namespace {
template <int CW>
__device__ __forceinline__ void ldv(const float* p, float* f) {
  if constexpr (CW == 4) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
  } else if constexpr (CW == 8) {
    ldv<4>(p, f);
    ldv<4>(p + 4, f + 4);
  } else {
    f[0] = *p;
  }
}
template <int CW>
__device__ __forceinline__ void ldv(const bf16_t* p, float* f) {
  if constexpr (CW == 4) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    f[0] = __uint_as_float(w.x << 16); f[1] = __uint_as_float(w.x & 0xffff0000u);
    f[2] = __uint_as_float(w.y << 16); f[3] = __uint_as_float(w.y & 0xffff0000u);
  } else if constexpr (CW == 8) {
    const uint4 w = *reinterpret_cast<const uint4*>(p);
    const uint32_t u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f[2 * i] = __uint_as_float(u[i] << 16);
      f[2 * i + 1] = __uint_as_float(u[i] & 0xffff0000u);
    }
  } else {
    f[0] = ldf(p);
  }
}
template <int CW>
__device__ __forceinline__ void stv(float* p, const float* f) {
  if constexpr (CW == 4) {
    *reinterpret_cast<float4*>(p) = make_float4(f[0], f[1], f[2], f[3]);
  } else if constexpr (CW == 8) {
    stv<4>(p, f);
    stv<4>(p + 4, f + 4);
  } else {
    *p = f[0];
  }
}
template <int CW>
__device__ __forceinline__ void stv(bf16_t* p, const float* f) {
  if constexpr (CW == 1) {
    stf(p, f[0]);
  } else {
    uint32_t u[CW / 2];
#pragma unroll
    for (int i = 0; i < CW / 2; ++i) {
      bf16_t lo, hi;
      stf(&lo, f[2 * i]);
      stf(&hi, f[2 * i + 1]);
      u[i] = (uint32_t)lo | ((uint32_t)hi << 16);
    }
    if constexpr (CW == 4) *reinterpret_cast<uint2*>(p) = make_uint2(u[0], u[1]);
    else *reinterpret_cast<uint4*>(p) = make_uint4(u[0], u[1], u[2], u[3]);
  }
}

// CW values at c of a row whose type is a runtime flag
template <int CW>
__device__ __forceinline__ void ld_flag(const void* p, bool f32, int64_t at, float* f) {
  if (f32) ldv<CW>(static_cast<const float*>(p) + at, f);
  else ldv<CW>(static_cast<const bf16_t*>(p) + at, f);
}
}  // namespace

struct GainRows {
  float* x;
  const void *y, *y2, *h_in;
  int64_t ys, y2s, hs;
  int y_f32, y2_f32, h_f32;
  const float* y2_logit;         // one per row, stride below
  int64_t ls;
  const float* h_weight;         // [T]
  float g_post, g_pre, eps;
  void* out;
  int T, d;
};

// NCH > 0: the row lives in registers, d <= NCH * 256 * CW; NCH == 0: any d, read twice.
template <typename TO, int CW, int NCH>
__global__ __launch_bounds__(256) void gain_sandwich_kernel(const GainRows a) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, d = a.d;
  float* xr = a.x + (int64_t)t * d;
  const float sg = a.y2 != nullptr ? 1.0f / (1.0f + expf(-a.y2_logit[(int64_t)t * a.ls])) : 0.f;
  const float hw = a.h_in != nullptr ? a.h_weight[t] : 0.f;
  auto sub = [&](int c, float* v) {
#pragma unroll
    for (int i = 0; i < CW; ++i) v[i] = 0.f;
    if (a.y != nullptr) ld_flag<CW>(a.y, a.y_f32, (int64_t)t * a.ys + c, v);
    float u[CW];
    if (a.y2 != nullptr) {
      ld_flag<CW>(a.y2, a.y2_f32, (int64_t)t * a.y2s + c, u);
#pragma unroll
      for (int i = 0; i < CW; ++i) v[i] += sg * u[i];
    }
    if (a.h_in != nullptr) {
      ld_flag<CW>(a.h_in, a.h_f32, (int64_t)t * a.hs + c, u);
#pragma unroll
      for (int i = 0; i < CW; ++i) v[i] += hw * u[i];
    }
  };
  const bool add = a.y != nullptr || a.y2 != nullptr || a.h_in != nullptr;
  TO* out = static_cast<TO*>(a.out) + (int64_t)t * d;
  if constexpr (NCH > 0) {
    float xv[NCH][CW], yv[NCH][CW];
    float sy = 0.f;
#pragma unroll
    for (int k = 0; k < NCH; ++k) {
      const int c = (threadIdx.x + k * 256) * CW;
      if (c < d) {
        ldv<CW>(xr + c, xv[k]);
        if (add) {
          sub(c, yv[k]);
#pragma unroll
          for (int i = 0; i < CW; ++i) sy += yv[k][i] * yv[k][i];
        }
      }
    }
    if (add) {
      sy = block_sum(sy, scratch);
      const float ry = a.g_post / sqrtf(sy / (float)d + a.eps);
#pragma unroll
      for (int k = 0; k < NCH; ++k) {
        const int c = (threadIdx.x + k * 256) * CW;
        if (c < d) {
#pragma unroll
          for (int i = 0; i < CW; ++i) xv[k][i] += yv[k][i] * ry;
          stv<CW>(xr + c, xv[k]);
        }
      }
    }
    if (a.out == nullptr) return;
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NCH; ++k)
      if ((int)(threadIdx.x + k * 256) * CW < d) {
#pragma unroll
        for (int i = 0; i < CW; ++i) ss += xv[k][i] * xv[k][i];
      }
    ss = block_sum(ss, scratch);
    const float r = a.g_pre / sqrtf(ss / (float)d + a.eps);
#pragma unroll
    for (int k = 0; k < NCH; ++k) {
      const int c = (threadIdx.x + k * 256) * CW;
      if (c < d) {
#pragma unroll
        for (int i = 0; i < CW; ++i) xv[k][i] *= r;
        stv<CW>(out + c, xv[k]);
      }
    }
  } else {
    float ss = 0.f;
    if (add) {
      float sy = 0.f;
      for (int c = threadIdx.x * CW; c < d; c += 256 * CW) {
        float v[CW];
        sub(c, v);
#pragma unroll
        for (int i = 0; i < CW; ++i) sy += v[i] * v[i];
      }
      sy = block_sum(sy, scratch);
      const float ry = a.g_post / sqrtf(sy / (float)d + a.eps);
      for (int c = threadIdx.x * CW; c < d; c += 256 * CW) {
        float v[CW], xv[CW];
        sub(c, v);
        ldv<CW>(xr + c, xv);
#pragma unroll
        for (int i = 0; i < CW; ++i) {
          xv[i] += v[i] * ry;
          ss += xv[i] * xv[i];
        }
        stv<CW>(xr + c, xv);
      }
    } else {
      for (int c = threadIdx.x * CW; c < d; c += 256 * CW) {
        float xv[CW];
        ldv<CW>(xr + c, xv);
#pragma unroll
        for (int i = 0; i < CW; ++i) ss += xv[i] * xv[i];
      }
    }
    if (a.out == nullptr) return;
    ss = block_sum(ss, scratch);
    const float r = a.g_pre / sqrtf(ss / (float)d + a.eps);
    for (int c = threadIdx.x * CW; c < d; c += 256 * CW) {      // own writes
      float xv[CW];
      ldv<CW>(xr + c, xv);
#pragma unroll
      for (int i = 0; i < CW; ++i) xv[i] *= r;
      stv<CW>(out + c, xv);
    }
  }
}

// ------------------------------------------------------------------ polynomial norm unit
__device__ __forceinline__ void block_sum3(float& a, float& b, float& c, float* scratch) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, nw = blockDim.x >> 6;
  a = wave_sum(a);
  b = wave_sum(b);
  c = wave_sum(c);
  if (lane == 0) {
    scratch[wid] = a;
    scratch[16 + wid] = b;
    scratch[32 + wid] = c;
  }
  __syncthreads();
  a = b = c = 0.f;
  for (int w = 0; w < nw; ++w) {
    a += scratch[w];
    b += scratch[16 + w];
    c += scratch[32 + w];
  }
}

// NCH > 0: F <= NCH * blockDim * CW, the row in registers; NCH == 0: read twice.
template <typename T, int CW, int NCH>
__global__ __launch_bounds__(NCH == 8 ? 512 : 1024) void poly_norm_rows_kernel(
    const T* x, int64_t xs, T* out, int64_t os, int F, float ca, float cb,
    float cc, float ce, float eps) {
  __shared__ float scratch[48];
  const int t = blockIdx.x, nthr = blockDim.x;
  const T* xr = x + (int64_t)t * xs;
  T* orow = out + (int64_t)t * os;
  float s2 = 0.f, s4 = 0.f, s6 = 0.f;
  float z[NCH > 0 ? NCH : 1][CW];
  auto sums = [&](const float* v) {
#pragma unroll
    for (int i = 0; i < CW; ++i) {
      const float q = v[i] * v[i];
      s2 += q;
      s4 += q * q;
      s6 += q * q * q;
    }
  };
  if constexpr (NCH > 0) {
#pragma unroll
    for (int k = 0; k < NCH; ++k) {
      const int c = (threadIdx.x + k * nthr) * CW;
      if (c < F) {
        ldv<CW>(xr + c, z[k]);
        sums(z[k]);
      }
    }
  } else {
    for (int c = threadIdx.x * CW; c < F; c += nthr * CW) {
      ldv<CW>(xr + c, z[0]);
      sums(z[0]);
    }
  }
  block_sum3(s2, s4, s6, scratch);
  const float n = 1.0f / (float)F;
  const float ra = ca / sqrtf(s2 * n + eps), rb = cb / sqrtf(s4 * n + eps),
              rc = cc / sqrtf(s6 * n + eps);
  auto unit = [&](float* v) {
#pragma unroll
    for (int i = 0; i < CW; ++i) v[i] = v[i] * (ra + v[i] * (rb + v[i] * rc)) + ce;
  };
  if constexpr (NCH > 0) {
#pragma unroll
    for (int k = 0; k < NCH; ++k) {
      const int c = (threadIdx.x + k * nthr) * CW;
      if (c < F) {
        unit(z[k]);
        stv<CW>(orow + c, z[k]);
      }
    }
  } else {
    for (int c = threadIdx.x * CW; c < F; c += nthr * CW) {
      ldv<CW>(xr + c, z[0]);
      unit(z[0]);
      stv<CW>(orow + c, z[0]);
    }
  }
}

// ------------------------------------------------------------------ launchers
namespace {
bool al(const void* p, int n) { return reinterpret_cast<uintptr_t>(p) % n == 0; }
}  // namespace

void launch_gain_sandwich(bool out_f32, float* x, const void* y, int64_t ys, bool y_f32,
                          const void* y2, int64_t y2s, bool y2_f32, const float* y2_logit,
                          int64_t ls, const void* h_in, int64_t hs, bool h_f32,
                          const float* h_weight, float g_post, float g_pre, float eps, void* out,
                          int T, int d, hipStream_t s) {
  if (T == 0) return;
  const GainRows a{x, y, y2, h_in, ys, y2s, hs, (int)y_f32, (int)y2_f32, (int)h_f32, y2_logit, ls,
                   h_weight, g_post, g_pre, eps, out, T, d};
  const bool vec = d % 4 == 0 && ys % 4 == 0 && y2s % 4 == 0 && hs % 4 == 0 && al(x, 16) &&
                   al(y, y_f32 ? 16 : 8) && al(y2, y2_f32 ? 16 : 8) && al(h_in, h_f32 ? 16 : 8) &&
                   al(out, out_f32 ? 16 : 8);
#define GAIN_GO(CW, NCH)                                                                           \
  do {                                                                                             \
    if (out_f32) hipLaunchKernelGGL((gain_sandwich_kernel<float, CW, NCH>), dim3(T), dim3(256), 0, s, a); \
    else hipLaunchKernelGGL((gain_sandwich_kernel<bf16_t, CW, NCH>), dim3(T), dim3(256), 0, s, a); \
  } while (0)
  if (!vec) GAIN_GO(1, 0);
  else if (d <= 1024) GAIN_GO(4, 1);
  else if (d <= 2048) GAIN_GO(4, 2);
  else if (d <= 4096) GAIN_GO(4, 4);
  else if (d <= 8192) GAIN_GO(4, 8);
  else GAIN_GO(4, 0);
#undef GAIN_GO
}

void launch_poly_norm_rows(bool f32, const void* x, int64_t xs, void* out, int64_t os, int T, int F,
                           float a, float b, float c, float e, float eps, hipStream_t s) {
  if (T == 0 || F == 0) return;
  const bool vec = F % 8 == 0 && xs % 8 == 0 && os % 8 == 0 && al(x, 16) && al(out, 16);
#define POLY_GO(CW, NCH, THREADS)                                                               \
  do {                                                                                          \
    if (f32)                                                                                    \
      hipLaunchKernelGGL((poly_norm_rows_kernel<float, CW, NCH>), dim3(T), dim3(THREADS), 0, s, \
                         (const float*)x, xs, (float*)out, os, F, a, b, c, e, eps);             \
    else                                                                                        \
      hipLaunchKernelGGL((poly_norm_rows_kernel<bf16_t, CW, NCH>), dim3(T), dim3(THREADS), 0, s, \
                         (const bf16_t*)x, xs, (bf16_t*)out, os, F, a, b, c, e, eps);           \
  } while (0)
  if (!vec) POLY_GO(1, 0, 256);
  else if (F <= 2048) POLY_GO(8, 1, 256);
  else if (F <= 4096) POLY_GO(8, 2, 256);
  else if (F <= 8192) POLY_GO(8, 4, 256);
  else if (F <= 16384) POLY_GO(8, 4, 512);
  else if (F <= 32768) POLY_GO(8, 8, 512);
  else POLY_GO(8, 0, 512);
#undef POLY_GO
}

}  // namespace rfqmix
