// Row kernels of layers around several residual streams:
//
//   streams_norm    x_t <- sum_s mix[s, t] x_s + w_out[t] y (the previous streams on the right),
//                   u = sum_s w_in[s] x_s and out = norm(u) w for the next sublayer (layer norm
//                   without bias, or RMS norm): one kernel per sublayer boundary.  The first one
//                   starts the streams from the embedding table, the last one need not write them.
//   gelu_glu_rows   g(gate) * up with the tanh form of gelu
//   gate_heads      [H, T, n] products of the heads laid side by side as [T, H n], times
//                   sigmoid(gate)
//
// Streams, sums and norms are fp32 whatever the activation type is.
#include "mix_common.h"

namespace rfqmix {

namespace {
constexpr int kMaxStreams = 16;

template <int CW>
__device__ __forceinline__ void ldv(const float* p, float* f) {
  static_assert(CW == 1 || CW == 4 || CW == 8, "width");
  if constexpr (CW == 1) {
    f[0] = *p;
  } else {
#pragma unroll
    for (int i = 0; i < CW; i += 4) {
      const float4 a = *reinterpret_cast<const float4*>(p + i);
      f[i] = a.x; f[i + 1] = a.y; f[i + 2] = a.z; f[i + 3] = a.w;
    }
  }
}
template <int CW>
__device__ __forceinline__ void ldv(const bf16_t* p, float* f) {
  if constexpr (CW == 1) {
    f[0] = ldf(p);
  } else {
    uint32_t u[CW / 2];
    if constexpr (CW == 4) {
      const uint2 w = *reinterpret_cast<const uint2*>(p);
      u[0] = w.x; u[1] = w.y;
    } else {
      const uint4 w = *reinterpret_cast<const uint4*>(p);
      u[0] = w.x; u[1] = w.y; u[2] = w.z; u[3] = w.w;
    }
#pragma unroll
    for (int i = 0; i < CW / 2; ++i) {
      f[2 * i] = __uint_as_float(u[i] << 16);
      f[2 * i + 1] = __uint_as_float(u[i] & 0xffff0000u);
    }
  }
}
template <int CW>
__device__ __forceinline__ void stv(float* p, const float* f) {
  if constexpr (CW == 1) {
    *p = f[0];
  } else {
#pragma unroll
    for (int i = 0; i < CW; i += 4)
      *reinterpret_cast<float4*>(p + i) = make_float4(f[i], f[i + 1], f[i + 2], f[i + 3]);
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
    if constexpr (CW == 4)
      *reinterpret_cast<uint2*>(p) = make_uint2(u[0], u[1]);
    else
      *reinterpret_cast<uint4*>(p) = make_uint4(u[0], u[1], u[2], u[3]);
  }
}
}  // namespace

// One workgroup per row.  S > 0: that many streams; S = 0: `streams` of them, at most
// kMaxStreams.  Every thread works on the same entries in all three passes, so the sublayer's input
// row u in LDS needs no barrier.  LDS: d floats.
template <typename T, int S, int CW>
__global__ __launch_bounds__(1024) void streams_norm_kernel(
    float* __restrict__ x, const int32_t* __restrict__ ids, const T* __restrict__ table, int vocab,
    const T* __restrict__ y, int64_t y_stride, const float* __restrict__ mix,
    const float* __restrict__ w_out, const float* __restrict__ w_in, const float* __restrict__ w,
    float eps, int centre, T* __restrict__ out, int d, int streams, int keep) {
  constexpr int N = S > 0 ? S : kMaxStreams;
  const int ns = S > 0 ? S : streams;
  extern __shared__ __attribute__((aligned(16))) float u_row[];
  __shared__ float scratch[16];
  const int t = blockIdx.x;
  float* xr = x + (int64_t)t * ns * d;
  const T* er = nullptr;
  if (ids != nullptr) {
    int id = ids[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    er = table + (int64_t)id * d;
  }
  const T* yr = y != nullptr ? y + (int64_t)t * y_stride : nullptr;
  const int step = blockDim.x * CW;
  float sum = 0.f;
  for (int c = threadIdx.x * CW; c < d; c += step) {
    float xs[N][CW], u[CW], yv[CW];
    if (er != nullptr) {
      ldv<CW>(er + c, xs[0]);
#pragma unroll
      for (int s = 1; s < N; ++s)
#pragma unroll
        for (int i = 0; i < CW; ++i) xs[s][i] = xs[0][i];
    } else {
#pragma unroll
      for (int s = 0; s < N; ++s)
        if (s < ns) ldv<CW>(xr + (int64_t)s * d + c, xs[s]);
    }
#pragma unroll
    for (int i = 0; i < CW; ++i) u[i] = 0.f;
    if (yr != nullptr) ldv<CW>(yr + c, yv);
#pragma unroll
    for (int o = 0; o < N; ++o) {
      if (o >= ns) break;
      float v[CW];
      if (yr != nullptr) {
        const float wo = w_out[o];
#pragma unroll
        for (int i = 0; i < CW; ++i) v[i] = wo * yv[i];
#pragma unroll
        for (int s = 0; s < N; ++s)
          if (s < ns) {
            const float ms = mix[s * ns + o];
#pragma unroll
            for (int i = 0; i < CW; ++i) v[i] += ms * xs[s][i];
          }
      } else {
#pragma unroll
        for (int i = 0; i < CW; ++i) v[i] = xs[o][i];
      }
      if (keep) stv<CW>(xr + (int64_t)o * d + c, v);
      const float wi = w_in[o];
#pragma unroll
      for (int i = 0; i < CW; ++i) u[i] += wi * v[i];
    }
    stv<CW>(u_row + c, u);
#pragma unroll
    for (int i = 0; i < CW; ++i) sum += u[i];
  }
  const float mean = centre ? block_sum(sum, scratch) / (float)d : 0.f;
  float ss = 0.f;
  for (int c = threadIdx.x * CW; c < d; c += step) {
    float u[CW];
    ldv<CW>(u_row + c, u);
#pragma unroll
    for (int i = 0; i < CW; ++i) ss += (u[i] - mean) * (u[i] - mean);
  }
  ss = block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)d + eps);
  for (int c = threadIdx.x * CW; c < d; c += step) {
    float u[CW], wv[CW];
    ldv<CW>(u_row + c, u);
    ldv<CW>(w + c, wv);
#pragma unroll
    for (int i = 0; i < CW; ++i) u[i] = (u[i] - mean) * r * wv[i];
    stv<CW>(out + (int64_t)t * d + c, u);
  }
}

// z / 2 (1 + tanh(a)) = z / (1 + exp(-2 a)), a = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh_f(float z, float /*fp32*/) {
  return z / (1.0f + expf(-1.5957691216057308f * (z + 0.044715f * z * z * z)));
}
__device__ __forceinline__ float gelu_tanh_f(float z, bf16_t) {
  return z * __builtin_amdgcn_rcpf(1.0f + __expf(-1.5957691216057308f * (z + 0.044715f * z * z * z)));
}

template <typename T, int CW>
__global__ __launch_bounds__(256) void gelu_glu_rows_kernel(const T* __restrict__ gu, int64_t gs,
                                                            T* __restrict__ out, int64_t os, int F) {
  const int t = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * CW;
  if (c >= F) return;
  float g[CW], u[CW];
  ldv<CW>(gu + (int64_t)t * gs + c, g);
  ldv<CW>(gu + (int64_t)t * gs + F + c, u);
#pragma unroll
  for (int i = 0; i < CW; ++i) g[i] = gelu_tanh_f(g[i], T(0)) * u[i];
  stv<CW>(out + (int64_t)t * os + c, g);
}

template <typename T, int CW>
__global__ __launch_bounds__(256) void gate_heads_kernel(
    const T* __restrict__ x, int64_t xh, int64_t xt, const T* __restrict__ gate, int64_t gs,
    T* __restrict__ out, int64_t os, int HN, int n) {
  const int t = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * CW;
  if (c >= HN) return;
  const int h = c / n, e = c - h * n;
  float v[CW], g[CW];
  ldv<CW>(x + h * xh + t * xt + e, v);
  ldv<CW>(gate + (int64_t)t * gs + c, g);
#pragma unroll
  for (int i = 0; i < CW; ++i) v[i] /= 1.0f + expf(-g[i]);
  stv<CW>(out + (int64_t)t * os + c, v);
}

// ------------------------------------------------------------------ launchers
namespace {
bool al16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

struct StreamsArgs {
  float* x;
  const int32_t* ids;
  const void* table;
  int vocab;
  const void* y;
  int64_t ys;
  const float *mix, *w_out, *w_in, *w;
  float eps;
  int centre;
  void* out;
  int T, d, streams, keep;
  hipStream_t s;
};

template <typename TT, int S, int CW>
void launch_streams_one(const StreamsArgs& a) {
  // few rows (decode): one pass over the row with up to 1024 threads; many rows: 256 each
  int threads = 256;
  if (a.T <= 1024) {
    const int need = (a.d / CW + 63) / 64 * 64;
    threads = need < 256 ? 256 : (need > 1024 ? 1024 : need);
  }
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&streams_norm_kernel<TT, S, CW>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, 159 * 1024);
    attr = true;
  }
  hipLaunchKernelGGL((streams_norm_kernel<TT, S, CW>), dim3(a.T), dim3(threads),
                     (size_t)a.d * sizeof(float), a.s, a.x, a.ids, (const TT*)a.table, a.vocab,
                     (const TT*)a.y, a.ys, a.mix, a.w_out, a.w_in, a.w, a.eps, a.centre, (TT*)a.out,
                     a.d, a.streams, a.keep);
}

template <typename TT, int CW>
void launch_streams_any(const StreamsArgs& a) {
  switch (a.streams) {
    case 1: launch_streams_one<TT, 1, CW>(a); break;
    case 2: launch_streams_one<TT, 2, CW>(a); break;
    case 3: launch_streams_one<TT, 3, CW>(a); break;
    case 4: launch_streams_one<TT, 4, CW>(a); break;
    default: launch_streams_one<TT, 0, CW>(a); break;
  }
}
}  // namespace

bool streams_norm_ok(int streams, int64_t d) {
  return streams >= 1 && streams <= kMaxStreams && d >= 1 && d * 4 <= 158 * 1024;
}

void launch_streams_norm(bool f32, float* x, const int32_t* ids, const void* table, int vocab,
                         const void* y, int64_t ys, const float* mix, const float* w_out,
                         const float* w_in, const float* w, float eps, bool centre, void* out, int T,
                         int d, int streams, bool keep, hipStream_t s) {
  if (T == 0) return;
  const StreamsArgs a{x, ids, table, vocab, y, ys, mix, w_out, w_in, w, eps, (int)centre, out, T, d,
                      streams, (int)keep, s};
  const bool vec = d % 4 == 0 && ys % 4 == 0 && al16(x) && al16(table) && al16(y) && al16(w) && al16(out);
  if (f32) {
    if (vec) launch_streams_any<float, 4>(a);
    else launch_streams_any<float, 1>(a);
  } else {
    if (vec) launch_streams_any<bf16_t, 4>(a);
    else launch_streams_any<bf16_t, 1>(a);
  }
}

void launch_gelu_glu_rows(bool f32, const void* gu, int64_t gs, void* out, int64_t os, int T, int F,
                          hipStream_t s) {
  if (T == 0 || F == 0) return;
  const bool vec = F % 8 == 0 && gs % 8 == 0 && os % 8 == 0 && al16(gu) && al16(out);
  const int per = vec ? 2048 : 256;
  const dim3 grid(T, (F + per - 1) / per);
#define GLU_GO(TT, CW)                                                                              \
  hipLaunchKernelGGL((gelu_glu_rows_kernel<TT, CW>), grid, dim3(256), 0, s, (const TT*)gu, gs,     \
                     (TT*)out, os, F)
  if (f32) {
    if (vec) GLU_GO(float, 8);
    else GLU_GO(float, 1);
  } else {
    if (vec) GLU_GO(bf16_t, 8);
    else GLU_GO(bf16_t, 1);
  }
#undef GLU_GO
}

void launch_gate_heads(bool f32, const void* x, int64_t xh, int64_t xt, const void* gate, int64_t gs,
                       void* out, int64_t os, int T, int H, int n, hipStream_t s) {
  if (T == 0) return;
  const int HN = H * n;
  const bool vec = n % 8 == 0 && xh % 8 == 0 && xt % 8 == 0 && gs % 8 == 0 && os % 8 == 0 && al16(x) &&
                   al16(gate) && al16(out);
  const int per = vec ? 2048 : 256;
  const dim3 grid(T, (HN + per - 1) / per);
#define GH_GO(TT, CW)                                                                              \
  hipLaunchKernelGGL((gate_heads_kernel<TT, CW>), grid, dim3(256), 0, s, (const TT*)x, xh, xt,    \
                     (const TT*)gate, gs, (TT*)out, os, HN, n)
  if (f32) {
    if (vec) GH_GO(float, 8);
    else GH_GO(float, 1);
  } else {
    if (vec) GH_GO(bf16_t, 8);
    else GH_GO(bf16_t, 1);
  }
#undef GH_GO
}

}  // namespace rfqmix
