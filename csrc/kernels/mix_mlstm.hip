// Matrix-memory recurrence with exponential gates, token by token (any sizes, either type).
//
// Per head a state S of dim key x vdim value channels, a key sum n and a running maximum m, all
// fp32 and zero at the start (m too):
//
//   li = cap tanh((zi + bi) / cap)          lf = log sigmoid(cap tanh((zf + bf) / cap))
//   m' = max(lf + m, li);  a = exp(lf + m - m');  b = exp(li - m')
//   S <- a S + b k v^T;  n <- a n + b k
//   o = S^T q / (max(|n . q|, exp(-m')) + 1e-6)              q already scaled
//   out = o / sqrt(mean(o^2) + eps) * norm_w * sigmoid(gate)
//
// Rows of a sequence are contiguous in a step (a "run").  row_state = slot * 2 + half to read
// (-1: none), row_back = index of the row inside its run, row_fwd = rows of the run after it.
// The state pools are double buffered: a run reads its sequence's half and writes the other,
// and a run that starts at position 0 reads nothing (the slot may hold another sequence's rest).
//
// One workgroup per (run, head, block of VW value channels).  Thread (r, c) holds rows
// r, r + R, ... of CW neighbouring columns of S in registers for the whole run; q, k and the
// key sum pass through LDS, the row groups' partial read-outs meet there.  Long steps leave norm
// and gate to a row-parallel kernel (raw read-outs); a bf16 model's long prompts run the chunked
// form of mix_mlstm_mfma.hip.
#include "mix_common.h"
#include "mix_mlstm.h"

namespace rfqmix {

namespace {
constexpr int kThreads = 256;
constexpr int kMaxDim = 1024;

__device__ __forceinline__ float log_sigmoid(float x) {
  return -(fmaxf(-x, 0.f) + log1pf(expf(-fabsf(x))));
}

template <int CW, typename T>
__device__ __forceinline__ void ld_cols(const T* p, float* f) {
  if constexpr (CW == 4 && sizeof(T) == 4) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w;
  } else if constexpr (CW == 4) {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    f[0] = __uint_as_float(w.x << 16); f[1] = __uint_as_float(w.x & 0xffff0000u);
    f[2] = __uint_as_float(w.y << 16); f[3] = __uint_as_float(w.y & 0xffff0000u);
  } else {
    f[0] = ldf(p);
  }
}
}  // namespace

// LDS (floats): qs[2][dim] | ks[2][dim] | ns[dim] | red[2][R VW] | den[2][4] | scratch[16]
// NQ: key channels per thread while q and k are loaded (dim <= NQ * 256)
template <typename T, int CW, int NA, int NQ>
__global__ __launch_bounds__(kThreads, NA <= 4 ? 5 : NA <= 8 ? 4 : 2) void mlstm_step_kernel(const MlstmArgs a, int VW, int R) {
  const int t0 = a.run_rows != nullptr ? a.run_rows[blockIdx.x] : (int)blockIdx.x;
  const int h = blockIdx.y;
  if (t0 < 0 || a.row_back[t0] != 0) return;
  const int n = a.row_fwd[t0] + 1;
  const int code = a.row_state[t0];
  const int dim = a.dim, vdim = a.vdim, H = a.H;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int VT = VW / CW;
  const int r = tid / VT, vt = tid - r * VT;
  const int c0 = (int)blockIdx.z * VW;                 // first value channel of the block
  const int col = c0 + vt * CW;
  const bool live = r < R && col < vdim;

  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* qs = lds;
  float* ks = qs + 2 * dim;
  float* ns = ks + 2 * dim;
  float* red = ns + dim;
  float* den = red + 2 * R * VW;
  float* scratch = den + 8;

  const bool from_state = code >= 0 && a.pos[t0] > 0;
  const int64_t rh = ((int64_t)(code & 1) * a.slots + (code >> 1)) * H + h;
  float s[NA][CW];
#pragma unroll
  for (int x = 0; x < NA; ++x) {
    const int i = r + R * x;
#pragma unroll
    for (int c = 0; c < CW; ++c) s[x][c] = 0.f;
    if (from_state && live && i < dim) ld_cols<CW>(a.S + (rh * dim + i) * vdim + col, s[x]);
  }
  for (int i = tid; i < dim; i += kThreads) ns[i] = from_state ? a.n[rh * dim + i] : 0.f;
  float m = from_state ? a.m[rh] : 0.f;

  const float bi = a.zbias[h], bf = a.zbias[H + h], cap = a.cap, icap = 1.0f / a.cap;
  const T* qp = static_cast<const T*>(a.q) + h * dim;
  const T* kp = static_cast<const T*>(a.k) + h * dim;
  const T* vp = static_cast<const T*>(a.v) + h * vdim + (live ? col : 0);
  float nq[NQ], nk[NQ], nv[CW], nzi, nzf;
  auto load = [&](int64_t t) {
#pragma unroll
    for (int x = 0; x < NQ; ++x) {
      const int i = tid + x * kThreads;
      if (i < dim) {
        nq[x] = ldf(qp + t * a.qs + i);
        nk[x] = ldf(kp + t * a.ks + i);
      }
    }
    if (live) ld_cols<CW>(vp + t * a.vs, nv);
    nzi = a.z[t * a.zs + h];
    nzf = a.z[t * a.zs + H + h];
  };
#pragma unroll
  for (int c = 0; c < CW; ++c) nv[c] = 0.f;
  load(t0);
  for (int x = 0; x < n; ++x) {
    const int b = x & 1;
#pragma unroll
    for (int y = 0; y < NQ; ++y) {
      const int i = tid + y * kThreads;
      if (i < dim) {
        qs[b * dim + i] = nq[y] * a.q_scale;
        ks[b * dim + i] = nk[y];
      }
    }
    float v[CW];
#pragma unroll
    for (int c = 0; c < CW; ++c) v[c] = nv[c];
    const float li = cap * tanhf((nzi + bi) * icap);
    const float lf = log_sigmoid(cap * tanhf((nzf + bf) * icap));
    __syncthreads();
    if (x + 1 < n) load((int64_t)t0 + x + 1);          // in flight during the sums
    const float mn = fmaxf(lf + m, li);
    const float keep = expf(lf + m - mn), add = expf(li - mn);
    m = mn;
    float acc[CW];
#pragma unroll
    for (int c = 0; c < CW; ++c) acc[c] = 0.f;
#pragma unroll
    for (int y = 0; y < NA; ++y) {
      const int i = r + R * y;
      if (i < dim && r < R) {
        const float kk = ks[b * dim + i] * add, qq = qs[b * dim + i];
#pragma unroll
        for (int c = 0; c < CW; ++c) {
          s[y][c] = keep * s[y][c] + kk * v[c];
          acc[c] += s[y][c] * qq;
        }
      }
    }
    float* rd = red + b * R * VW;
    if (r < R) {
#pragma unroll
      for (int c = 0; c < CW; ++c) rd[r * VW + vt * CW + c] = acc[c];
    }
    float dn = 0.f;
    for (int i = tid; i < dim; i += kThreads) {
      const float u = keep * ns[i] + add * ks[b * dim + i];
      ns[i] = u;
      dn += u * qs[b * dim + i];
    }
    dn = wave_sum(dn);
    if (lane == 0) den[b * 4 + wid] = dn;
    __syncthreads();
    const float* d4 = den + b * 4;
    const float dd = fmaxf(fabsf((d4[0] + d4[1]) + (d4[2] + d4[3])), expf(-m)) + 1e-6f;
    const int64_t t = (int64_t)t0 + x;
    const bool mine = tid < VW && c0 + tid < vdim;      // VW <= kThreads
    float o = 0.f;
    if (mine) {
      for (int y = 0; y < R; ++y) o += rd[y * VW + tid];
      o /= dd;
    }
    const int64_t at = (int64_t)h * vdim + c0 + tid;
    if (a.raw != nullptr) {
      if (mine) a.raw[t * H * vdim + at] = o;
      continue;
    }
    const float ss = block_sum(o * o, scratch);          // one block holds the whole head here
    if (mine) {
      const float g = ldf(static_cast<const T*>(a.gate) + t * a.gs + at);
      stf(static_cast<T*>(a.out) + t * H * vdim + at,
          o / sqrtf(ss / (float)vdim + a.eps) * a.norm_w[at] / (1.0f + expf(-g)));
    }
  }
  if (code < 0) return;
  const int64_t wh = ((int64_t)(1 - (code & 1)) * a.slots + (code >> 1)) * H + h;
  if (live) {
#pragma unroll
    for (int x = 0; x < NA; ++x) {
      const int i = r + R * x;
      if (i < dim) {
        float* w = a.S + (wh * dim + i) * vdim + col;
        if constexpr (CW == 4)
          *reinterpret_cast<float4*>(w) = make_float4(s[x][0], s[x][1], s[x][2], s[x][3]);
        else
          *w = s[x][0];
      }
    }
  }
  if (blockIdx.z == 0) {
    for (int i = tid; i < dim; i += kThreads) a.n[wh * dim + i] = ns[i];   // own writes
    if (tid == 0) a.m[wh] = m;
  }
}

// out = raw / sqrt(mean(raw^2) + eps) * norm_w * sigmoid(gate), a wave per (row, head).
template <typename T>
__global__ __launch_bounds__(256) void mlstm_finish_kernel(
    const float* __restrict__ raw, const T* __restrict__ gate, int64_t gs,
    const float* __restrict__ norm_w, float eps, T* __restrict__ out, int rows, int H, int vdim) {
  const int lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  if (item >= (int64_t)rows * H) return;
  const int64_t t = item / H;
  const int h = (int)(item - t * H);
  const float* r = raw + item * vdim;
  float ss = 0.f;
  for (int c = lane; c < vdim; c += 64) ss += r[c] * r[c];
  ss = wave_sum(ss);
  const float inv = 1.0f / sqrtf(ss / (float)vdim + eps);
  for (int c = lane; c < vdim; c += 64) {
    const float g = ldf(gate + t * gs + (int64_t)h * vdim + c);
    stf(out + item * vdim + c, r[c] * inv * norm_w[h * vdim + c] / (1.0f + expf(-g)));
  }
}

// ------------------------------------------------------------------ launchers
namespace {
struct StepPlan {
  int CW, VW, R, NA, blocks;
};
// The widest block of value channels whose state fits 16 registers per column and thread.
StepPlan plan_step(int dim, int vdim, bool vec) {
  StepPlan p{};
  p.CW = vec ? 4 : 1;
  for (int nb = 1; nb <= vdim; ++nb) {
    int VW = (vdim + nb - 1) / nb;
    VW = (VW + p.CW - 1) / p.CW * p.CW;
    if (VW > kThreads) continue;
    const int VT = VW / p.CW;
    int R = kThreads / VT;
    if (R > dim) R = dim;
    const int NA = (dim + R - 1) / R;
    if (NA <= 16) {
      p.VW = VW;
      p.R = R;
      p.NA = NA;
      p.blocks = (vdim + VW - 1) / VW;
      return p;
    }
  }
  return p;                                             // blocks 0: not reached for dim <= 1024
}
size_t step_lds(int dim, const StepPlan& p) {
  return (size_t)(5 * dim + 2 * p.R * p.VW + 8 + 16) * sizeof(float);     // < 64 KB
}
}  // namespace

bool mlstm_ok(int dim, int vdim) {
  return dim >= 1 && dim <= kMaxDim && vdim >= 1 && vdim <= 65535;
}

void launch_mlstm_finish(bool f32, const MlstmArgs& a, hipStream_t s) {
  const int64_t items = (int64_t)a.T * a.H;
  if (items == 0) return;
  const dim3 grid((unsigned)((items + 3) / 4));
  if (f32)
    hipLaunchKernelGGL(mlstm_finish_kernel<float>, grid, dim3(256), 0, s, a.raw,
                       (const float*)a.gate, a.gs, a.norm_w, a.eps, (float*)a.out, a.T, a.H, a.vdim);
  else
    hipLaunchKernelGGL(mlstm_finish_kernel<bf16_t>, grid, dim3(256), 0, s, a.raw,
                       (const bf16_t*)a.gate, a.gs, a.norm_w, a.eps, (bf16_t*)a.out, a.T, a.H,
                       a.vdim);
}

// Whether one block holds a head's value channels, so that norm and gate can be fused; else the
// caller brings `raw`.
bool mlstm_fuses(int dim, int vdim, bool vec) { return plan_step(dim, vdim, vec).blocks == 1; }

bool mlstm_vec(bool f32, const MlstmArgs& a) {
  const int w = f32 ? 16 : 8;
  return a.vdim % 4 == 0 && a.vs % 4 == 0 && reinterpret_cast<uintptr_t>(a.v) % w == 0 &&
         reinterpret_cast<uintptr_t>(a.S) % 16 == 0;
}

void launch_mlstm(bool f32, const MlstmArgs& a, hipStream_t s) {
  if (a.T == 0 || (a.run_rows != nullptr && a.runs == 0)) return;
  const StepPlan p = plan_step(a.dim, a.vdim, mlstm_vec(f32, a));
  const size_t lds = step_lds(a.dim, p);
  const dim3 grid(a.run_rows != nullptr ? a.runs : a.T, a.H, p.blocks);
#define MLSTM_GO(TT, CW, NA)                                                                      \
  do {                                                                                            \
    if (a.dim <= kThreads)                                                                        \
      hipLaunchKernelGGL((mlstm_step_kernel<TT, CW, NA, 1>), grid, dim3(kThreads), lds, s, a,     \
                         p.VW, p.R);                                                              \
    else                                                                                          \
      hipLaunchKernelGGL((mlstm_step_kernel<TT, CW, NA, kMaxDim / kThreads>), grid, dim3(kThreads), \
                         lds, s, a, p.VW, p.R);                                                   \
  } while (0)
#define MLSTM_NA(TT, CW)                     \
  do {                                       \
    if (p.NA <= 2) MLSTM_GO(TT, CW, 2);      \
    else if (p.NA <= 4) MLSTM_GO(TT, CW, 4); \
    else if (p.NA <= 8) MLSTM_GO(TT, CW, 8); \
    else MLSTM_GO(TT, CW, 16);               \
  } while (0)
  if (f32) {
    if (p.CW == 4) MLSTM_NA(float, 4);
    else MLSTM_NA(float, 1);
  } else {
    if (p.CW == 4) MLSTM_NA(bf16_t, 4);
    else MLSTM_NA(bf16_t, 1);
  }
#undef MLSTM_NA
#undef MLSTM_GO
  if (a.raw != nullptr) launch_mlstm_finish(f32, a, s);
}

}  // namespace rfqmix
