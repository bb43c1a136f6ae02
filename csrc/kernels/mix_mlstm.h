// Arguments of the matrix-memory recurrence's launchers (mix_mlstm.hip, mix_mlstm_mfma.hip),
// shared with the bindings.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace rfqmix {

struct MlstmArgs {
  const void *q, *k, *v;            // [T, H dim] x2, [T, H vdim]; row strides below
  int64_t qs, ks, vs;
  const float* z;                   // raw gate logits [T, i: H | f: H]
  int64_t zs;
  const float* zbias;               // [2 H]
  float cap, q_scale;
  const void* gate;                 // [T, H vdim]
  int64_t gs;
  const float* norm_w;              // [H vdim]
  float eps;
  float* raw;                       // [T, H vdim] fp32 or null: read-outs before norm and gate
  float *S, *n, *m;                 // [2 slots, H, dim, vdim], [2 slots, H, dim], [2 slots, H]
  const int32_t *row_state, *row_back, *row_fwd, *pos, *run_rows;
  int runs;
  void* out;                        // [T, H vdim]
  int T, H, dim, vdim, slots;
};

bool mlstm_ok(int dim, int vdim);
bool mlstm_chunk_ok(int dim, int vdim);
void launch_mlstm(bool f32, const MlstmArgs& a, hipStream_t s);
bool launch_mlstm_chunk(const MlstmArgs& a, hipStream_t s);     // bf16, needs raw
void launch_mlstm_finish(bool f32, const MlstmArgs& a, hipStream_t s);

}  // namespace rfqmix
