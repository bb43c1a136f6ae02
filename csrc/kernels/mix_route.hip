// Mixture of experts with grouped sigmoid routing or grouped softmax routing with identity
// experts, any sizes, either activation type.  Sigmoid routing:
//
//   s = sigmoid(z)                       router scores (z: fp32 router logits)
//   choice = s + correction              chooses; the weights use s
//   groups: `groups` equal groups of neighbouring experts, a group's score = the sum of its two
//           largest choice scores; only experts of the `keep` best groups can be chosen
//   weights = s[chosen] / (sum + 1e-20)
//
// The expert products here are the general path: one (token, choice) pair per workgroup
// streams its expert's rows (weights stay in L2 between pairs of the same expert).  Steps of
// bf16 models whose sizes fit the grouped MFMA GEMMs use those instead.
#include "mix_common.h"

namespace rfqmix {

constexpr float kNegInfR = -__builtin_huge_valf();

// One thread per token.  Ties go to the lower index (strict comparisons, ascending scans).
__global__ __launch_bounds__(256) void moe_route_grouped_kernel(
    const float* __restrict__ z, const float* __restrict__ corr, int T, int E, int top, int groups,
    int keep, int32_t* __restrict__ ids, float* __restrict__ weights) {
  const int t = blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= T) return;
  const float* zr = z + (int64_t)t * E;
  int32_t* id = ids + (int64_t)t * top;
  float* wt = weights + (int64_t)t * top;
  uint64_t kept = ~0ull;
  int per = E;
  if (groups > 0) {
    per = E / groups;
    kept = 0;
    for (int a = 0; a < keep; ++a) {
      int best = -1;
      float bs = 0.f;
      for (int g = 0; g < groups; ++g) {
        if ((kept >> g) & 1) continue;
        float m1 = kNegInfR, m2 = kNegInfR;
        for (int e = g * per; e < (g + 1) * per; ++e) {
          const float c = 1.0f / (1.0f + expf(-zr[e])) + corr[e];
          if (c > m1) { m2 = m1; m1 = c; } else if (c > m2) { m2 = c; }
        }
        const float sc = per > 1 ? m1 + m2 : m1;
        if (best < 0 || sc > bs) { best = g; bs = sc; }
      }
      kept |= 1ull << best;
    }
  }
  float sum = 0.f;
  for (int a = 0; a < top; ++a) {
    int best = -1;
    float bc = 0.f, bsc = 0.f;
    for (int e = 0; e < E; ++e) {
      if (groups > 0 && !((kept >> (e / per)) & 1)) continue;
      bool used = false;
      for (int b = 0; b < a; ++b) used |= id[b] == e;
      if (used) continue;
      const float s = 1.0f / (1.0f + expf(-zr[e]));
      const float c = s + corr[e];
      if (best < 0 || c > bc) { best = e; bc = c; bsc = s; }
    }
    id[a] = best;
    wt[a] = bsc;
    sum += bsc;
  }
  const float inv = 1.0f / (sum + 1e-20f);
  for (int a = 0; a < top; ++a) wt[a] *= inv;
}

// Softmax routing over `real` experts followed by identity experts (whose output is their input),
// n = E columns of z in all:
//   s = softmax(z);  choice = s + correction (chooses; the weights use s)
//   a group's score is its largest choice score; only the `keep` best of `groups` equal groups of
//   neighbours can be chosen (groups 0: no limit)
//   weights = scale * s[chosen], not renormalised
// A chosen identity expert is written as id `real` with weight 0 (a segment no expert kernel
// computes) and its weight is added to ident[t].  One wave per token: a lane holds columns lane,
// lane + 64, ...; ties go to the lower index.  LDS: choice[E] | s[E] | group[groups].
__global__ __launch_bounds__(64) void moe_route_softmax_kernel(
    const float* __restrict__ z, int64_t zs, const float* __restrict__ corr, int E, int real,
    int top, int groups, int keep, float scale, int32_t* __restrict__ ids,
    float* __restrict__ weights, float* __restrict__ ident) {
  extern __shared__ float lds[];
  float* ch = lds;
  float* sc = ch + E;
  float* gr = sc + E;
  const int t = blockIdx.x, lane = threadIdx.x;
  const float* zr = z + (int64_t)t * zs;
  float mx = kNegInfR;
  for (int e = lane; e < E; e += 64) mx = fmaxf(mx, zr[e]);
  mx = wave_max(mx);
  float sum = 0.f;
  for (int e = lane; e < E; e += 64) {
    const float p = expf(zr[e] - mx);
    sc[e] = p;
    sum += p;
  }
  const float inv = 1.0f / wave_sum(sum);
  for (int e = lane; e < E; e += 64) {
    const float p = sc[e] * inv;
    sc[e] = p;
    ch[e] = p + corr[e];
  }
  __syncthreads();
  // the largest of v[0 .. n) in every lane (index n: nothing left); taken ones are -inf
  auto best_of = [&](const float* v, int n) {
    float b = kNegInfR;
    int bi = n;
    for (int e = lane; e < n; e += 64)
      if (v[e] > b) {
        b = v[e];
        bi = e;
      }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(b, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ob > b || (ob == b && oi < bi)) {
        b = ob;
        bi = oi;
      }
    }
    return bi;
  };
  if (groups > 0) {
    const int per = E / groups;
    for (int g = lane; g < groups; g += 64) {
      float m = kNegInfR;
      for (int e = g * per; e < (g + 1) * per; ++e) m = fmaxf(m, ch[e]);
      gr[g] = m;
    }
    __syncthreads();
    uint64_t kept[4] = {0, 0, 0, 0};                   // groups <= 256
    for (int a = 0; a < keep; ++a) {
      const int g = best_of(gr, groups);
      if (g < groups) {
#pragma unroll
        for (int w = 0; w < 4; ++w)
          if ((g >> 6) == w) kept[w] |= 1ull << (g & 63);
        if (lane == 0) gr[g] = kNegInfR;
      }
      __syncthreads();
    }
    for (int e = lane; e < E; e += 64) {
      const int g = e / per;
      uint64_t w = kept[0];
#pragma unroll
      for (int k = 1; k < 4; ++k)
        if ((g >> 6) == k) w = kept[k];
      if (!((w >> (g & 63)) & 1)) ch[e] = kNegInfR;
    }
    __syncthreads();
  }
  float id_sum = 0.f;
  for (int a = 0; a < top; ++a) {
    const int e = best_of(ch, E);
    const bool any = e < E;                            // non-finite logits: nothing to choose
    const bool is_real = any && e < real;
    const float w = any ? sc[e] * scale : 0.f;
    if (any && !is_real) id_sum += w;
    if (lane == 0) {
      ids[(int64_t)t * top + a] = is_real ? e : real;
      weights[(int64_t)t * top + a] = is_real ? w : 0.f;
    }
    __syncthreads();
    if (lane == 0 && any) ch[e] = kNegInfR;
    __syncthreads();
  }
  if (lane == 0 && ident != nullptr) ident[t] = id_sum;
}

// act[p, f] = silu(Wg[e] . x_t) * (Wu[e] . x_t) for pair p = t * top + k, e = ids[p].
// Grid (pairs, feature tiles of FT); x_t staged in LDS as floats; one wave per feature.
template <typename T>
__global__ __launch_bounds__(256) void moe_pair_up_kernel(
    const T* __restrict__ h, int64_t h_stride, const int32_t* __restrict__ ids,
    const T* __restrict__ w13, T* __restrict__ act, int top, int d, int F, int E, int FT) {
  extern __shared__ float xs[];
  const int p = blockIdx.x, t = p / top;
  const int e = ids[p];
  if (e < 0 || e >= E) return;
  for (int c = threadIdx.x; c < d; c += blockDim.x) xs[c] = ldf(h + (int64_t)t * h_stride + c);
  __syncthreads();
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const T* wg = w13 + (int64_t)e * 2 * F * d;
  const int f1 = min(F, (blockIdx.y + 1) * FT);
  for (int f = blockIdx.y * FT + wid; f < f1; f += nw) {
    const T* g = wg + (int64_t)f * d;
    const T* u = wg + (int64_t)(F + f) * d;
    float ag = 0.f, au = 0.f;
    for (int c = lane; c < d; c += 64) {
      const float x = xs[c];
      ag += ldf(g + c) * x;
      au += ldf(u + c) * x;
    }
    ag = wave_sum(ag);
    au = wave_sum(au);
    if (lane == 0) stf(act + (int64_t)p * F + f, ag / (1.0f + expf(-ag)) * au);
  }
}

// out[t, c] = base[t, c] + sum_k weights[t, k] * (W2[ids[t, k]][c, :] . act[t * top + k, :]).
// Grid (tokens, column tiles of CT); the token's `top` activation rows staged in LDS.
template <typename T>
__global__ __launch_bounds__(256) void moe_pair_down_kernel(
    const T* __restrict__ act, const int32_t* __restrict__ ids, const float* __restrict__ weights,
    const T* __restrict__ w2, const T* __restrict__ base, int64_t base_stride,
    float* __restrict__ out, int top, int d, int F, int E, int CT) {
  extern __shared__ float as[];                // [top][F]
  const int t = blockIdx.x;
  for (int x = threadIdx.x; x < top * F; x += blockDim.x)
    as[x] = ldf(act + (int64_t)t * top * F + x);
  __syncthreads();
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, nw = blockDim.x >> 6;
  const int c1 = min(d, (blockIdx.y + 1) * CT);
  for (int c = blockIdx.y * CT + wid; c < c1; c += nw) {
    float acc = 0.f;
    for (int k = 0; k < top; ++k) {
      const int e = ids[(int64_t)t * top + k];
      if (e < 0 || e >= E) continue;
      const T* row = w2 + ((int64_t)e * d + c) * F;
      const float* a = as + k * F;
      float dot = 0.f;
      for (int f = lane; f < F; f += 64) dot += ldf(row + f) * a[f];
      acc += weights[(int64_t)t * top + k] * dot;
    }
    acc = wave_sum(acc);
    if (lane == 0)
      out[(int64_t)t * d + c] = acc + (base != nullptr ? ldf(base + (int64_t)t * base_stride + c) : 0.f);
  }
}

// ------------------------------------------------------------------ launchers
void launch_moe_route_grouped(const float* z, const float* corr, int T, int E, int top, int groups,
                              int keep, int32_t* ids, float* weights, hipStream_t s) {
  if (T == 0) return;
  hipLaunchKernelGGL(moe_route_grouped_kernel, dim3((T + 255) / 256), dim3(256), 0, s, z, corr, T,
                     E, top, groups, keep, ids, weights);
}

bool moe_route_softmax_ok(int E, int groups) { return E <= 4096 && groups <= 256; }

void launch_moe_route_softmax(const float* z, int64_t zs, const float* corr, int T, int E, int real,
                              int top, int groups, int keep, float scale, int32_t* ids,
                              float* weights, float* ident, hipStream_t s) {
  if (T == 0) return;
  const size_t lds = (size_t)(2 * E + groups) * 4;
  hipLaunchKernelGGL(moe_route_softmax_kernel, dim3(T), dim3(64), lds, s, z, zs, corr, E, real, top,
                     groups, keep, scale, ids, weights, ident);
}

void launch_moe_pair_up(bool f32, const void* h, int64_t h_stride, const int32_t* ids,
                        const void* w13, void* act, int pairs, int top, int d, int F, int E,
                        hipStream_t s) {
  if (pairs == 0) return;
  const int FT = 64;
  const dim3 grid(pairs, (F + FT - 1) / FT);
  const size_t lds = (size_t)d * 4;
  if (f32)
    hipLaunchKernelGGL(moe_pair_up_kernel<float>, grid, dim3(256), lds, s, (const float*)h,
                       h_stride, ids, (const float*)w13, (float*)act, top, d, F, E, FT);
  else
    hipLaunchKernelGGL(moe_pair_up_kernel<bf16_t>, grid, dim3(256), lds, s, (const bf16_t*)h,
                       h_stride, ids, (const bf16_t*)w13, (bf16_t*)act, top, d, F, E, FT);
}

void launch_moe_pair_down(bool f32, const void* act, const int32_t* ids, const float* weights,
                          const void* w2, const void* base, int64_t base_stride, float* out, int T,
                          int top, int d, int F, int E, hipStream_t s) {
  if (T == 0) return;
  const int CT = 64;
  const dim3 grid(T, (d + CT - 1) / CT);
  const size_t lds = (size_t)top * F * 4;
  static bool attr = false;
  if (!attr) {
    hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_pair_down_kernel<float>),
                        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    hipFuncSetAttribute(reinterpret_cast<const void*>(&moe_pair_down_kernel<bf16_t>),
                        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    attr = true;
  }
  if (f32)
    hipLaunchKernelGGL(moe_pair_down_kernel<float>, grid, dim3(256), lds, s, (const float*)act, ids,
                       weights, (const float*)w2, (const float*)base, base_stride, out, top, d, F,
                       E, CT);
  else
    hipLaunchKernelGGL(moe_pair_down_kernel<bf16_t>, grid, dim3(256), lds, s, (const bf16_t*)act,
                       ids, weights, (const bf16_t*)w2, (const bf16_t*)base, base_stride, out, top,
                       d, F, E, CT);
}

}  // namespace rfqmix
