// Weight re-layout for the matrix-core linears; launched by the host library at compile() time.
#include <hip/hip_runtime.h>
#include <stdint.h>
#include "mk_types.h"

typedef unsigned u32x4 __attribute__((ext_vector_type(4)));

// Re-lays the weights of one linear stage in matrix-core tile order (MkStage::wpack); one thread per 16-byte operand.
// Rows past the last output repeat it (their products are never stored).
extern "C" __global__ __launch_bounds__(256) void mk_pack_weights_kernel(const MkWeight w, int n, int k, int silu, int half, u32x4 *dst, long long total) {
  const int k8 = k / 8, nsteps = k >> 6;
  const int n_out = silu ? n / 2 : n;
  for (long long idx = (long long)blockIdx.x * 256 + threadIdx.x; idx < total; idx += (long long)gridDim.x * 256) {
    const int lane = (int)(idx & 63);
    long long r = idx >> 6;
    const int h = (int)(r & 1);
    r >>= 1;
    const int step = (int)(r % nsteps), ti = (int)(r / nsteps);
    const int lr = lane & 15, lg = lane >> 4;
    int vr;
    if (silu) {
      const int o = min((ti >> 1) * 16 + lr, n_out - 1), gi = o / half;
      vr = gi * 2 * half + (o - gi * half) + ((ti & 1) ? half : 0);
    } else {
      vr = min(ti * 16 + lr, n_out - 1);
    }
    const u32x4 *row;
    if (w.nseg == 1) {
      row = (const u32x4 *)w.seg[0] + (size_t)vr * k8;
    } else {
      const int g = vr / w.group_rows;
      int o = vr - g * w.group_rows, sg = 0;
      while (sg + 1 < w.nseg && o >= w.seg_rows[sg]) o -= w.seg_rows[sg++];
      row = (const u32x4 *)w.seg[sg] + (size_t)(g * w.seg_rows[sg] + o) * k8;
    }
    dst[idx] = row[step * 8 + h * 4 + lg];
  }
}
