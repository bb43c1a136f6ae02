// Matrix-memory recurrence of mix_mlstm.hip in chunks of 64 tokens on MFMA tiles (bf16 operands,
// key width a multiple of 32, value width a multiple of 16).
//
// Inside a chunk, with b_t the running sum of the log forget gates, g_s = li_s - b_s and
// M_t = max(m, max_{s<=t} g_s) (m: the running maximum the chunk starts from), the recurrence is
//
//   m_t = b_t + M_t
//   o_t = [ e^{m - M_t} S^T q_t + sum_{s<=t} e^{g_s - M_t} (k_s . q_t) v_s ] / den_t
//   den_t = max(| e^{m - M_t} n . q_t + sum_{s<=t} e^{g_s - M_t} (k_s . q_t) |, e^{-m_t}) + 1e-6
//   S <- e^{m - M_L} S + sum_s e^{g_s - M_L} k_s v_s^T ;  n likewise with k alone ;  m <- m_L
//
// so a chunk is four products and the state advances once per chunk.  q, k and v enter as the
// bf16 numbers they are; the weights, the state and the weighted values are fp32 and enter the
// products as bf16 hi + lo parts (two MFMAs); n . q is summed in fp32.  b, g and M are formed in
// double and kept as two floats each, so that long runs of strong forgetting cancel exactly.
//
// One workgroup per (run, head, 64 value channels), four waves: in the read-out a wave takes 16
// queries, in the update 16 value channels; the fp32 state lives in the update's accumulators.
#include "common.h"
#include "mix_common.h"
#include "mix_mlstm.h"

namespace rfqmix {

using rfq::as_bf16x8;
using rfq::f32x4;
using rfq::s16x4;
using rfq::s16x8;

namespace {
constexpr int CL = 64;                  // tokens per chunk
constexpr int CV = 64;                  // value channels per workgroup
constexpr int CVR = CV + 8;             // shorts per value row in LDS
constexpr float kGone = -1e30f;         // log weight of a token that is not there

__device__ __forceinline__ void split8(const float* f, s16x8& hi, s16x8& lo) {
  float r[8];
  hi = rfq::pack8(f);
#pragma unroll
  for (int i = 0; i < 8; ++i) r[i] = f[i] - rfq::bf2f_s(hi[i]);
  lo = rfq::pack8(r);
}

template <int DI>
constexpr size_t chunk_lds() {
  return (size_t)(2 * CL * (16 * DI + 8) + CL * CVR + 2 * CV * (16 * DI + 8)) * 2 +
         (size_t)(16 * DI + 256 + 7 * CL + 2) * 4;
}
}  // namespace

// DI = dim / 16
template <int DI>
__global__ __launch_bounds__(256) void mlstm_chunk_kernel(const MlstmArgs a) {
  constexpr int dim = 16 * DI, DK = DI / 2, RS = dim + 8;
  const int t0 = a.run_rows != nullptr ? a.run_rows[blockIdx.x] : (int)blockIdx.x;
  const int h = blockIdx.y;
  if (t0 < 0 || a.row_back[t0] != 0) return;
  const int n = a.row_fwd[t0] + 1;
  const int code = a.row_state[t0];
  const int H = a.H, vdim = a.vdim;
  const int tid = threadIdx.x, lane = tid & 63, wid = tid >> 6;
  const int col = lane & 15, grp = lane >> 4;
  const int v0 = (int)blockIdx.z * CV;                 // first value channel of the workgroup

  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  short* Qs = reinterpret_cast<short*>(smem);          // [CL][RS]
  short* Ks = Qs + CL * RS;                            // [CL][RS]
  short* Vs = Ks + CL * RS;                            // [CL][CVR]
  short* Sh = Vs + CL * CVR;                           // [CV][RS]: S^T, high parts
  short* Sl = Sh + CV * RS;                            // [CV][RS]: low parts
  float* ns = reinterpret_cast<float*>(Sl + CV * RS);  // [dim]
  float* np = ns + dim;                                // [256] partial key sums
  float* gh = np + 256;                                // [CL] each from here on
  float* gl = gh + CL;
  float* Mh = gl + CL;
  float* Ml = Mh + CL;
  float* fac = Ml + CL;
  float* eneg = fac + CL;
  float* wts = eneg + CL;
  float* ctl = wts + CL;                               // [2]: keep factor, next maximum

  const bool from_state = code >= 0 && a.pos[t0] > 0;
  const int64_t rh = ((int64_t)(code & 1) * a.slots + (code >> 1)) * H + h;
  const int dv = v0 + 16 * wid + col;                  // this lane's value channel in the update
  f32x4 st[DI];                                        // S[16 ti + 4 grp + r][dv]
#pragma unroll
  for (int ti = 0; ti < DI; ++ti) {
    st[ti] = (f32x4){0.f, 0.f, 0.f, 0.f};
    if (from_state && dv < vdim) {
#pragma unroll
      for (int r = 0; r < 4; ++r) st[ti][r] = a.S[(rh * dim + 16 * ti + 4 * grp + r) * vdim + dv];
    }
  }
  auto stage_state = [&]() {
#pragma unroll
    for (int ti = 0; ti < DI; ++ti) {
      short hi[4], lo[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        bf16_t x, y;
        stf(&x, st[ti][r]);
        stf(&y, st[ti][r] - rfq::bf2f_s((short)x));
        hi[r] = (short)x;
        lo[r] = (short)y;
      }
      const int at = (16 * wid + col) * RS + 16 * ti + 4 * grp;
      *reinterpret_cast<s16x4*>(Sh + at) = (s16x4){hi[0], hi[1], hi[2], hi[3]};
      *reinterpret_cast<s16x4*>(Sl + at) = (s16x4){lo[0], lo[1], lo[2], lo[3]};
    }
  };
  stage_state();
  if (tid < dim) ns[tid] = from_state ? a.n[rh * dim + tid] : 0.f;
  float m = from_state ? a.m[rh] : 0.f;

  const bf16_t* qp = static_cast<const bf16_t*>(a.q) + h * dim;
  const bf16_t* kp = static_cast<const bf16_t*>(a.k) + h * dim;
  const bf16_t* vp = static_cast<const bf16_t*>(a.v) + (int64_t)h * vdim + v0;
  const float bi = a.zbias[h], bf = a.zbias[H + h], cap = a.cap, icap = 1.0f / a.cap;
  constexpr int NQ = CL * dim / 8 / 256, NV = CL * CV / 8 / 256;
  s16x8 qr[NQ], kr[NQ], vr[NV];
  float zi = 0.f, zf = 0.f;
  const s16x8 zero8 = (s16x8){0, 0, 0, 0, 0, 0, 0, 0};
  auto fetch = [&](int c0) {                           // rows c0 .. c0 + CL of the run; zeros past its end
#pragma unroll
    for (int x = 0; x < NQ; ++x) {
      const int p = tid + x * 256, row = p / (dim / 8), c = p - row * (dim / 8);
      qr[x] = kr[x] = zero8;
      if (c0 + row < n) {
        const int64_t t = (int64_t)t0 + c0 + row;
        qr[x] = *reinterpret_cast<const s16x8*>(qp + t * a.qs + c * 8);
        kr[x] = *reinterpret_cast<const s16x8*>(kp + t * a.ks + c * 8);
      }
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int p = tid + x * 256, row = p >> 3, c = p & 7;
      vr[x] = zero8;
      if (c0 + row < n && v0 + c * 8 < vdim)
        vr[x] = *reinterpret_cast<const s16x8*>(vp + ((int64_t)t0 + c0 + row) * a.vs + c * 8);
    }
    if (wid == 0 && c0 + lane < n) {
      const float* zr = a.z + ((int64_t)t0 + c0 + lane) * a.zs;
      zi = zr[h];
      zf = zr[H + h];
    }
  };
  fetch(0);
  float keep = 1.f;
  constexpr int PT = 256 / dim, PL = CL / PT;          // token parts of the key sum (dim 96: two)
  for (int c0 = 0; c0 < n; c0 += CL) {
    const int nrow = min(CL, n - c0);
    // ---- the chunk into LDS; the last chunk's key sum folded in; gates scanned by wave 0
#pragma unroll
    for (int x = 0; x < NQ; ++x) {
      const int p = tid + x * 256, row = p / (dim / 8), c = p - row * (dim / 8);
      *reinterpret_cast<s16x8*>(Qs + row * RS + c * 8) = qr[x];
      *reinterpret_cast<s16x8*>(Ks + row * RS + c * 8) = kr[x];
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int p = tid + x * 256, row = p >> 3, c = p & 7;
      *reinterpret_cast<s16x8*>(Vs + row * CVR + c * 8) = vr[x];
    }
    if (c0 > 0 && tid < dim) {
      float u = keep * ns[tid];
#pragma unroll
      for (int p = 0; p < PT; ++p) u += np[p * dim + tid];
      ns[tid] = u;
    }
    if (wid == 0) {
      const bool on = lane < nrow;
      const float li = cap * tanhf((zi + bi) * icap);
      const float fx = cap * tanhf((zf + bf) * icap);
      const float lf = -(fmaxf(-fx, 0.f) + log1pf(expf(-fabsf(fx))));
      double b = on ? (double)lf : 0.0;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double y = __shfl_up(b, o, 64);
        if (lane >= o) b += y;
      }
      const double g = on ? (double)li - b : (double)kGone;
      double M = g;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double y = __shfl_up(M, o, 64);
        if (lane >= o) M = fmax(M, y);
      }
      M = fmax(M, (double)m);
      const double Mlast = __shfl(M, 63, 64);
      const float g1 = (float)g, M1 = (float)M;
      gh[lane] = g1;
      gl[lane] = (float)(g - (double)g1);
      Mh[lane] = M1;
      Ml[lane] = (float)(M - (double)M1);
      fac[lane] = expf((float)((double)m - M)) * a.q_scale;
      eneg[lane] = expf((float)(-(b + M)));
      wts[lane] = expf((float)(g - Mlast));
      if (lane == 63) {
        ctl[0] = expf((float)((double)m - Mlast));
        ctl[1] = (float)(b + M);
      }
    }
    __syncthreads();
    if (c0 + CL < n) fetch(c0 + CL);                   // in flight during the products
    // ---- read-out: this wave's 16 queries
    const int tq = 16 * wid + col;
    if (16 * wid < nrow) {                             // wave-uniform
      s16x8 qf[DK];
      float nq = 0.f;
#pragma unroll
      for (int ks = 0; ks < DK; ++ks) {
        qf[ks] = *reinterpret_cast<const s16x8*>(Qs + tq * RS + ks * 32 + grp * 8);
#pragma unroll
        for (int j = 0; j < 8; ++j) nq += rfq::bf2f_s(qf[ks][j]) * ns[ks * 32 + grp * 8 + j];
      }
      nq += __shfl_xor(nq, 16, 64);
      nq += __shfl_xor(nq, 32, 64);
      f32x4 o[4];
      const float f = fac[tq];
#pragma unroll
      for (int mt = 0; mt < 4; ++mt) {
        o[mt] = (f32x4){0.f, 0.f, 0.f, 0.f};
        const int at = (16 * mt + col) * RS + grp * 8;
#pragma unroll
        for (int ks = 0; ks < DK; ++ks) {
          const s16x8 hi = *reinterpret_cast<const s16x8*>(Sh + at + ks * 32);
          const s16x8 lo = *reinterpret_cast<const s16x8*>(Sl + at + ks * 32);
          o[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(hi), as_bf16x8(qf[ks]), o[mt], 0, 0, 0);
          o[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(lo), as_bf16x8(qf[ks]), o[mt], 0, 0, 0);
        }
        o[mt] *= f;
      }
      const float mh = Mh[tq], ml = Ml[tq];
      float den = 0.f;
      for (int kp2 = 0; kp2 <= (wid >> 1); ++kp2) {    // 32 keys at a time, up to the queries'
        f32x4 sc[2];
        float pv[8];
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
          sc[kt] = (f32x4){0.f, 0.f, 0.f, 0.f};
          const short* kr2 = Ks + (kp2 * 32 + kt * 16 + col) * RS + grp * 8;
#pragma unroll
          for (int ks = 0; ks < DK; ++ks)
            sc[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                as_bf16x8(*reinterpret_cast<const s16x8*>(kr2 + ks * 32)), as_bf16x8(qf[ks]), sc[kt], 0, 0, 0);
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int s = kp2 * 32 + kt * 16 + grp * 4 + i;
            const float w = s <= tq ? __expf((gh[s] - mh) + (gl[s] - ml)) : 0.f;
            pv[kt * 4 + i] = sc[kt][i] * a.q_scale * w;
            den += pv[kt * 4 + i];
          }
        }
        s16x8 phi, plo;
        split8(pv, phi, plo);
        const short* u0 = Vs + (kp2 * 32 + 4 * grp + (col >> 2)) * CVR + 4 * (col & 3);
        const short* u1 = u0 + 16 * CVR;
#pragma unroll
        for (int mt = 0; mt < 4; ++mt) {
          const s16x4 x0 = rfq::ds_read_tr16(u0 + 16 * mt);
          const s16x4 x1 = rfq::ds_read_tr16(u1 + 16 * mt);
          const s16x8 x = (s16x8){x0[0], x0[1], x0[2], x0[3], x1[0], x1[1], x1[2], x1[3]};
          o[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(x), as_bf16x8(phi), o[mt], 0, 0, 0);
          o[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(x), as_bf16x8(plo), o[mt], 0, 0, 0);
        }
      }
      den += __shfl_xor(den, 16, 64);
      den += __shfl_xor(den, 32, 64);
      den = fmaxf(fabsf(den + nq * f), eneg[tq]) + 1e-6f;
      if (tq < nrow) {
        const float inv = 1.0f / den;
        float* orow = a.raw + ((int64_t)t0 + c0 + tq) * H * vdim + (int64_t)h * vdim + v0 + 4 * grp;
#pragma unroll
        for (int mt = 0; mt < 4; ++mt)
          if (v0 + 16 * mt + 4 * grp < vdim)
            *reinterpret_cast<float4*>(orow + 16 * mt) =
                make_float4(o[mt][0] * inv, o[mt][1] * inv, o[mt][2] * inv, o[mt][3] * inv);
      }
    }
    keep = ctl[0];
    m = ctl[1];
    __syncthreads();                                   // the state's readers are done
    // ---- update: this wave's 16 value channels; k slot (grp, j) of a 32-token step is token
    // 4 grp + j (j < 4) or 16 + 4 grp + j - 4 in both operands
    s16x8 vh[2], vl[2];
#pragma unroll
    for (int k2 = 0; k2 < 2; ++k2) {
      const short* u0 = Vs + (k2 * 32 + 4 * grp + (col >> 2)) * CVR + 4 * (col & 3) + 16 * wid;
      const s16x4 x0 = rfq::ds_read_tr16(u0), x1 = rfq::ds_read_tr16(u0 + 16 * CVR);
      float f8[8];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        f8[j] = rfq::bf2f_s(x0[j]) * wts[k2 * 32 + 4 * grp + j];
        f8[4 + j] = rfq::bf2f_s(x1[j]) * wts[k2 * 32 + 16 + 4 * grp + j];
      }
      split8(f8, vh[k2], vl[k2]);
    }
#pragma unroll
    for (int ti = 0; ti < DI; ++ti) {
      st[ti] *= keep;
#pragma unroll
      for (int k2 = 0; k2 < 2; ++k2) {
        const short* u0 = Ks + (k2 * 32 + 4 * grp + (col >> 2)) * RS + 4 * (col & 3) + 16 * ti;
        const s16x4 x0 = rfq::ds_read_tr16(u0), x1 = rfq::ds_read_tr16(u0 + 16 * RS);
        const s16x8 x = (s16x8){x0[0], x0[1], x0[2], x0[3], x1[0], x1[1], x1[2], x1[3]};
        st[ti] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(x), as_bf16x8(vh[k2]), st[ti], 0, 0, 0);
        st[ti] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(x), as_bf16x8(vl[k2]), st[ti], 0, 0, 0);
      }
    }
    stage_state();
    if (tid < PT * dim) {
      const int i = tid % dim, p = tid / dim;
      float u = 0.f;
#pragma unroll 8
      for (int s = p * PL; s < (p + 1) * PL; ++s) u += wts[s] * rfq::bf2f_s(Ks[s * RS + i]);
      np[p * dim + i] = u;
    }
    __syncthreads();
  }
  if (code < 0) return;
  const int64_t wh = ((int64_t)(1 - (code & 1)) * a.slots + (code >> 1)) * H + h;
  if (dv < vdim) {
#pragma unroll
    for (int ti = 0; ti < DI; ++ti)
#pragma unroll
      for (int r = 0; r < 4; ++r) a.S[(wh * dim + 16 * ti + 4 * grp + r) * vdim + dv] = st[ti][r];
  }
  if (blockIdx.z == 0) {
    if (tid < dim) {
      float u = keep * ns[tid];
#pragma unroll
      for (int p = 0; p < PT; ++p) u += np[p * dim + tid];
      a.n[wh * dim + tid] = u;
    }
    if (tid == 0) a.m[wh] = m;
  }
}

// ------------------------------------------------------------------ launcher
bool mlstm_chunk_ok(int dim, int vdim) {
  return (dim == 32 || dim == 64 || dim == 96 || dim == 128 || dim == 256) && vdim >= 16 &&
         vdim % 16 == 0;
}

template <int DI>
static void launch_mlstm_chunk_one(const MlstmArgs& a, hipStream_t s) {
  static bool attr = false;
  if (!attr) {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&mlstm_chunk_kernel<DI>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    attr = true;
  }
  const dim3 grid(a.run_rows != nullptr ? a.runs : a.T, a.H, (a.vdim + CV - 1) / CV);
  hipLaunchKernelGGL(mlstm_chunk_kernel<DI>, grid, dim3(256), chunk_lds<DI>(), s, a);
}

// False: sizes or alignments outside the tiles (the caller runs the token-by-token kernel).
bool launch_mlstm_chunk(const MlstmArgs& a, hipStream_t s) {
  if (!mlstm_chunk_ok(a.dim, a.vdim) || a.raw == nullptr) return false;
  auto al16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (a.qs % 8 || a.ks % 8 || a.vs % 8 || !al16(a.q) || !al16(a.k) || !al16(a.v) || !al16(a.raw))
    return false;
  if (a.T == 0 || (a.run_rows != nullptr && a.runs == 0)) return true;
  if (a.dim == 32) launch_mlstm_chunk_one<2>(a, s);
  else if (a.dim == 64) launch_mlstm_chunk_one<4>(a, s);
  else if (a.dim == 96) launch_mlstm_chunk_one<6>(a, s);
  else if (a.dim == 128) launch_mlstm_chunk_one<8>(a, s);
  else launch_mlstm_chunk_one<16>(a, s);
  launch_mlstm_finish(false, a, s);
  return true;
}

}  // namespace rfqmix
