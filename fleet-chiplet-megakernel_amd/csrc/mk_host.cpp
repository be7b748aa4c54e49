// Host side of the persistent decode megakernel: records the PersistentKernel task
// list, lowers it to the stage program the kernel walks, owns intermediate tensors
// and runtime state, and launches the kernel cooperatively.
//
// Replaces, for the decode path: src/kernel/graph.cc (register_task, attach_*,
// shuffle_tensors), src/kernel/task_register.cc (per-task validation),
// src/kernel/runtime.cc (register_mugraph / print_task_graph) and the host half of
// include/mirage/persistent_kernel/persistent_kernel.cuh:1960-2429.
#include <hip/hip_runtime.h>
#include <math.h>
#include <stdarg.h>
#include <stdio.h>
#include <stdlib.h>
#include <string.h>

#include <array>
#include <map>
#include <numeric>
#include <string>
#include <vector>

#include "../../include/fleet_mk.h"
#include "mk_types.h"

typedef unsigned u32x4 __attribute__((ext_vector_type(4)));

// the kernels, each from a translation unit of its own (build.py); a library may be built without some of them
extern "C" __global__ void mk_pack_weights_kernel(const MkWeight w, int n, int k, int silu, int half, u32x4 *dst, long long total);
#define MK_DECLARE_KERNEL(name) extern "C" __global__ void name(const MkRuntime rt, const MkRuntime *rtp, int max_iters, int run_scheduler)
#ifdef MK_HAVE_KERNEL_DENSE
MK_DECLARE_KERNEL(mk_persistent_kernel);
MK_DECLARE_KERNEL(mk_persistent_kernel_m1);
#endif
#ifdef MK_HAVE_KERNEL_FLEX
MK_DECLARE_KERNEL(mk_persistent_kernel_flex);
#endif
#ifdef MK_HAVE_KERNEL_FLEX_M1
MK_DECLARE_KERNEL(mk_persistent_kernel_flex_m1);
#endif
#ifdef MK_HAVE_KERNEL_FLEX_F32
MK_DECLARE_KERNEL(mk_persistent_kernel_flex_f32);
#endif
#ifdef MK_HAVE_KERNEL_MIX
MK_DECLARE_KERNEL(mk_persistent_kernel_mix);
#endif
#ifdef MK_HAVE_KERNEL_MIX_M1
MK_DECLARE_KERNEL(mk_persistent_kernel_mix_m1);
#endif
#ifdef MK_HAVE_KERNEL_MIX_F32
MK_DECLARE_KERNEL(mk_persistent_kernel_mix_f32);
#endif
#ifdef MK_HAVE_KERNEL_HYB
MK_DECLARE_KERNEL(mk_persistent_kernel_hyb);
#endif
#ifdef MK_HAVE_KERNEL_HYB_M1
MK_DECLARE_KERNEL(mk_persistent_kernel_hyb_m1);
#endif
#ifdef MK_HAVE_KERNEL_HYB_F32
MK_DECLARE_KERNEL(mk_persistent_kernel_hyb_f32);
#endif
#ifdef MK_HAVE_KERNEL_DUAL
MK_DECLARE_KERNEL(mk_persistent_kernel_dual);
#endif
#ifdef MK_HAVE_KERNEL_DUAL_M1
MK_DECLARE_KERNEL(mk_persistent_kernel_dual_m1);
#endif
#ifdef MK_HAVE_KERNEL_DUAL_F32
MK_DECLARE_KERNEL(mk_persistent_kernel_dual_f32);
#endif

namespace {

thread_local std::string g_err;

int fail(int code, const char *fmt, ...) {
  char buf[1024];
  va_list ap;
  va_start(ap, fmt);
  vsnprintf(buf, sizeof(buf), fmt, ap);
  va_end(ap);
  g_err = buf;
  return code;
}

#define HIP_TRY(expr)                                                                         \
  do {                                                                                        \
    hipError_t e_ = (expr);                                                                   \
    if (e_ != hipSuccess) return fail(MK_EHIP, "%s failed: %s", #expr, hipGetErrorString(e_)); \
  } while (0)

enum TensorKind { T_ATTACHED, T_OWNED, T_SHUFFLED };
enum FlexKind { FLEX_NONE, FLEX_BF16, FLEX_F32 };  // which stage set (and activation type) a graph runs on

struct Tensor {
  std::string name;
  int ndims = 0;
  int64_t dims[4] = {1, 1, 1, 1};
  int64_t strides[4] = {1, 1, 1, 1};
  int dtype = MK_DT_BF16;
  TensorKind kind = T_ATTACHED;
  void *ptr = nullptr;
  std::vector<int> sources;  // T_SHUFFLED
  int num_groups = 1;
  bool interleave = true;
  int io_category = 0;
  size_t elems() const {
    size_t n = 1;
    for (int i = 0; i < ndims; i++) n *= (size_t)dims[i];
    return n;
  }
};

struct Task {
  std::string name;
  int grid[3], block[3];
  std::vector<int> ops;
  std::vector<std::array<int, 3>> maps;
  std::vector<int> forloop;
  std::vector<int> params;
};

size_t dtype_size(int dt) {
  switch (dt) {
    case MK_DT_BF16:
    case MK_DT_F16: return 2;
    case MK_DT_F32:
    case MK_DT_I32: return 4;
    case MK_DT_I64:
    case MK_DT_U64: return 8;
    default: return 0;
  }
}

}  // namespace

struct mk_graph {
  mk_config cfg;
  int num_cus = 0;
  int G = 0;
  std::vector<Tensor> tensors;
  std::vector<Task> tasks;
  std::vector<Task> ltasks;  // what lower() walks: `tasks` with composite tasks expanded
  bool compiled = false;
  bool host_only = false;  // created with device < 0: records, validates, lowers and emits the task graph, never launches
  std::vector<void *> allocs;
  std::vector<void *> host_allocs;
  std::vector<MkStage> stages;
  std::vector<std::string> stage_desc;
  MkRuntime h_rt;
  MkRuntime *d_rt = nullptr;
  MkStage *d_stages = nullptr;
  MkSync *d_sync = nullptr;
  MkSched *d_sched = nullptr;
  long long *d_timing = nullptr;
  int timing_cap = 0;
  std::string json, program_text;
  hipEvent_t ev0 = nullptr, ev1 = nullptr;
  bool launch_pending = false;
  MkSync *pending_sync = nullptr;  // barrier state of the pending / last launch (the graph's own or the static scratch)
  int max_kv_heads = 1, max_qpk = 1;  // over the attention stages
  double last_ms = 0.0;
  int last_nxcd = 0, last_aborted = 0;
  int64_t weight_bytes = 0;
  int64_t packed_bytes = 0;  // matrix-core copies of the weights held by the handle
  size_t attn_cnt_n = 0;
  int num_ref_tasks = 0, num_ref_events = 0;
  int last_linear_task = -1, last_linear_stage = -1;  // lowering: the most recent linear task and the stage it became
  std::vector<int> stage_weight;      // per stage: tensor id of a LINEAR stage's weight operand (-1: none)
  std::vector<char> releasable;       // per tensor (single-weight-copy graphs, after mk_compile): the handle never reads it again
  bool single_copy = false;
  int spec_len = 0;  // guesses per decoding request (set by a find_ngram_global task)
  void *profiler_ptr = nullptr;  // the caller's profiler tensor (mk_set_profiler)
  long long profiler_cap = 0;
  int64_t row_major_bytes = 0;
  int flex = FLEX_NONE;
  size_t flex_items = 0;     // most work items of a flex attention stage (row tiles x kv heads x value slices)
  size_t flex_part = 0;      // floats of split-KV partials the flex and latent attention stages need
  bool mix = false;          // some stage is one of mk_mix.hip's
  bool hyb = false;          // ... of mk_hybrid.hip's, or an older stage has an option only the hybrid kernels know
  bool dual = false;         // ... of mk_dual.hip's, or an older stage has an option only the dual kernels know
  int *state_ids = nullptr;  // batch slot -> recurrent-state slot (the caller's tensor); null: no recurrence
};

namespace {

int dev_alloc(mk_graph *g, void **out, size_t bytes, bool zero = true) {
  if (bytes == 0) bytes = 16;
  if (g->host_only) {  // stand-in address: only its identity matters to the lowering
    *out = malloc(16);
    if (!*out) return fail(MK_EINVAL, "out of host memory");
    g->host_allocs.push_back(*out);
    return MK_OK;
  }
  HIP_TRY(hipMalloc(out, bytes));
  g->allocs.push_back(*out);
  if (zero) HIP_TRY(hipMemset(*out, 0, bytes));
  return MK_OK;
}

bool is_norm(const std::string &n) { return n == "rmsnorm" || n == "gang_rmsnorm_mi300"; }

// Classify linear-type task names: returns false if `n` is not a linear.
bool linear_kind(const std::string &n, bool *res, bool *silu, int *n_extra_inputs) {
  *res = false;
  *silu = false;
  *n_extra_inputs = 0;
  static const char *plain[] = {"linear", "gang_linear_mi300", "gang_linear_n_tiling_mi300", "gang_linear_msplit_mi300",
                                "splitk_linear_mi300"};
  static const char *with_res[] = {"linear_with_residual", "gang_linear_res_mi300", "gang_linear_res_n_tiling_mi300",
                                   "gang_linear_res_msplit_mi300"};
  static const char *fused_silu[] = {"linear_silu_mi300", "gang_linear_silu_mi300"};
  for (auto p : plain)
    if (n == p) return true;
  for (auto p : with_res)
    if (n == p) {
      *res = true;
      return true;
    }
  for (auto p : fused_silu)
    if (n == p) {
      *silu = true;
      return true;
    }
  if (n == "splitk_linear_res_atomic_mi300") {  // [input, weight, residual, workspace, done_counter, output]
    *res = true;
    *n_extra_inputs = 2;
    return true;
  }
  if (n == "gang_splitk_linear_res_mi300") {  // [input, weight, residual, workspace, output]
    *res = true;
    *n_extra_inputs = 1;
    return true;
  }
  return false;
}

int resolve_weight(mk_graph *g, int id, int64_t k, MkWeight *w, int64_t *rows_out, int *group_half, int dtype = MK_DT_BF16) {
  const Tensor &t = g->tensors[id];
  memset(w, 0, sizeof(*w));
  if (t.ndims != 2) return fail(MK_EINVAL, "weight '%s' must be 2-D", t.name.c_str());
  if (t.dtype != dtype) return fail(MK_EINVAL, "weight '%s' must be %s", t.name.c_str(), dtype == MK_DT_F32 ? "fp32, like the activations" : "bf16");
  if (t.dims[1] != k) return fail(MK_EINVAL, "weight '%s' has k=%lld, expected %lld", t.name.c_str(), (long long)t.dims[1], (long long)k);
  *rows_out = t.dims[0];
  *group_half = 0;
  if (t.kind != T_SHUFFLED) {
    if (!t.ptr) return fail(MK_EINVAL, "weight '%s' has no storage", t.name.c_str());
    w->nseg = 1;
    w->seg[0] = t.ptr;
    w->seg_rows[0] = (int)t.dims[0];
    w->group_rows = (int)t.dims[0];
    return MK_OK;
  }
  const int n = (int)t.sources.size();
  if (n > MK_MAX_SEGS) return fail(MK_EUNSUPPORTED, "shuffled weight '%s' has %d sources (max %d)", t.name.c_str(), n, MK_MAX_SEGS);
  int groups = t.interleave ? t.num_groups : 1;
  int total = 0;
  for (int i = 0; i < n; i++) {
    const Tensor &s = g->tensors[t.sources[i]];
    if (s.kind == T_SHUFFLED || !s.ptr) return fail(MK_EINVAL, "source '%s' of '%s' has no storage", s.name.c_str(), t.name.c_str());
    if (s.dims[0] % groups) return fail(MK_EINVAL, "source '%s' rows %lld not divisible by %d groups", s.name.c_str(), (long long)s.dims[0], groups);
    w->seg[i] = s.ptr;
    w->seg_rows[i] = (int)(s.dims[0] / groups);
    total += w->seg_rows[i];
  }
  w->nseg = n;
  w->group_rows = total;
  if (n == 2 && w->seg_rows[0] == w->seg_rows[1]) *group_half = w->seg_rows[0];
  return MK_OK;
}

std::string fmt(const char *f, ...) {
  char buf[512];
  va_list ap;
  va_start(ap, f);
  vsnprintf(buf, sizeof(buf), f, ap);
  va_end(ap);
  return buf;
}

// operands are listed inputs first, outputs last: how many of a task's operands are outputs
int num_outputs(const Task &t) {
  if (t.name == "argmax_partial") return 2;
  if (t.name == "gang_attn_split_kv_mi300") return 3;
  if (t.name == "paged_attention_ck_fmha_split_kv_mi300" || t.name == "paged_attention_split_kv_mi300") return 2;
  if (t.name == "moe_topk_softmax_mi300") return 3;
  if (t.name == "embedding_scaled" || t.name == "residual_rmsnorm" || t.name == "residual_prenorm" || t.name == "latent_prep" || t.name == "general_delta" || t.name == "expert_route" || t.name == "ring_conv") return 2;
  return 1;
}

// constants of the flex tasks travel as the bits of a float in an int parameter
float bits_f32(int bits) {
  float f;
  memcpy(&f, &bits, sizeof(f));
  return f;
}

bool rows_ok(const Tensor &t, int B, int64_t cols, int dtype) { return t.ndims == 2 && t.dims[0] >= B && t.dims[1] >= cols && t.dtype == dtype && !(t.strides[0] & 3); }
bool vector_ok(const Tensor &t, int64_t n) { return t.dtype == MK_DT_F32 && (int64_t)t.elems() >= n; }

// a graph holds flex stages of one activation type, and none of the fixed-shape stages next to them (checked after lowering)
int set_flex(mk_graph *g, int dtype, const char *task) {
  const int kind = dtype == MK_DT_F32 ? FLEX_F32 : FLEX_BF16;
  if (dtype != MK_DT_F32 && dtype != MK_DT_BF16) return fail(MK_EINVAL, "task '%s': activations must be bf16 or fp32", task);
  if (g->flex != FLEX_NONE && g->flex != kind) return fail(MK_EINVAL, "task '%s': the graph mixes bf16 and fp32 activations", task);
  g->flex = kind;
  return MK_OK;
}

// Lower one linear-type task (optionally preceded by a norm task whose output it consumes, optionally
// followed by a silu_mul consuming its output) into stages.
int lower_linear(mk_graph *g, size_t &i) {
  const Task *norm = nullptr;
  if (is_norm(g->ltasks[i].name)) {
    norm = &g->ltasks[i];
    i++;
  }
  const Task &lt = g->ltasks[i];
  bool res, silu;
  int extra;
  if (!linear_kind(lt.name, &res, &silu, &extra)) return fail(MK_EINVAL, "internal: '%s' is not a linear", lt.name.c_str());
  const size_t need_ops = 3 + (res ? 1 : 0) + extra;
  if (lt.ops.size() != need_ops) return fail(MK_EINVAL, "task '%s' expects %zu operands, got %zu", lt.name.c_str(), need_ops, lt.ops.size());
  const int in_id = lt.ops[0], w_id = lt.ops[1];
  int res_id = res ? lt.ops[2] : -1, out_id = lt.ops.back();
  size_t consumed_linear = 1;
  if (lt.name == "splitk_linear_mi300" && g->tensors[out_id].dtype == MK_DT_F32) {
    // the reference's two-task split-K: partial products into an fp32 workspace, then splitk_reduce [workspace, residual,
    // output] sums the slices and adds the residual.  The pair is one stage here; the workspace is never written.
    const Task *rd = i + 1 < g->ltasks.size() ? &g->ltasks[i + 1] : nullptr;
    if (!rd || rd->name != "splitk_reduce_mi300" || rd->ops.size() != 3 || rd->ops[0] != out_id)
      return fail(MK_EUNSUPPORTED, "splitk_linear_mi300 into an fp32 workspace must be followed by splitk_reduce_mi300 over that workspace");
    res = true;
    res_id = rd->ops[1];
    out_id = rd->ops[2];
    consumed_linear = 2;
  }
  const Tensor &tin = g->tensors[in_id];
  Tensor &tout = g->tensors[out_id];
  if (tin.ndims != 2 || tout.ndims != 2) return fail(MK_EINVAL, "task '%s': input/output must be 2-D", lt.name.c_str());
  const bool f32 = tin.dtype == MK_DT_F32;  // 32-bit linear: plain or SwiGLU, part of a flex graph
  if (tin.dtype != tout.dtype || (tin.dtype != MK_DT_BF16 && (!f32 || res || norm))) return fail(MK_EINVAL, "task '%s': activations must be bf16", lt.name.c_str());
  if (f32) {
    int rc = set_flex(g, MK_DT_F32, lt.name.c_str());
    if (rc) return rc;
  }
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = f32 ? MK_OP_LINEAR_F32 : MK_OP_LINEAR;
  st.k = (int)tin.dims[1];
  if (st.k % 8) return fail(MK_EINVAL, "task '%s': reduction length %d must be a multiple of 8", lt.name.c_str(), st.k);
  if (g->cfg.max_num_batched_tokens > 1 && st.k % 32) return fail(MK_EINVAL, "task '%s': reduction length %d must be a multiple of 32 when more than one token is batched", lt.name.c_str(), st.k);
  int64_t rows;
  int half;
  int rc = resolve_weight(g, w_id, st.k, &st.w, &rows, &half, tin.dtype);
  if (rc) return rc;
  st.n = (int)rows;
  st.eps = g->cfg.rms_eps;
  // a following silu_mul over this linear's (library-owned) output is folded into the epilogue
  const Task *act = nullptr;
  const bool gelu = i + 1 < g->ltasks.size() && g->ltasks[i + 1].name == "gelu_mul";
  if (!silu && !res && i + 1 < g->ltasks.size() && (gelu || g->ltasks[i + 1].name == "silu_mul") && g->ltasks[i + 1].ops.size() == 2 &&
      g->ltasks[i + 1].ops[0] == out_id && tout.kind == T_OWNED) {
    act = &g->ltasks[i + 1];
  }
  int final_out = out_id;
  const Task *sq = nullptr;  // a following relu_squared likewise
  if (!silu && !res && i + 1 < g->ltasks.size() && g->ltasks[i + 1].name == "relu_squared" && g->ltasks[i + 1].ops.size() == 2 && g->ltasks[i + 1].ops[0] == out_id && tout.kind == T_OWNED) {
    sq = &g->ltasks[i + 1];
    st.flags |= MK_F_RELU2;
    final_out = sq->ops[1];
    g->mix = g->hyb = true;
    int rc2 = set_flex(g, tin.dtype, "relu_squared");
    if (rc2) return rc2;
  }
  if (silu || act) {
    st.flags |= MK_F_SILU;
    if (act && gelu) {
      st.flags |= MK_F_GELU;
      g->mix = g->hyb = g->dual = true;
      int rc2 = set_flex(g, tin.dtype, "gelu_mul");
      if (rc2) return rc2;
    }
    if (act) {
      final_out = act->ops[1];
      const int groups = act->grid[0] * act->grid[1] * act->grid[2];
      if (groups <= 0 || (rows / 2) % groups) return fail(MK_EINVAL, "silu_mul grid %d does not divide %lld outputs", groups, (long long)(rows / 2));
      st.silu_half = (int)(rows / 2 / groups);
    } else {
      st.silu_half = half ? half : 128;  // physically interleaved weight: reference layout [gate128 ; up128]
    }
    if (half && half != st.silu_half) return fail(MK_EINVAL, "task '%s': shuffled group half %d != activation half %d", lt.name.c_str(), half, st.silu_half);
    if (rows % (2 * st.silu_half)) return fail(MK_EINVAL, "task '%s': %lld rows not a multiple of %d", lt.name.c_str(), (long long)rows, 2 * st.silu_half);
  }
  const Tensor &tfo = g->tensors[final_out];
  const int n_out = (st.flags & MK_F_SILU) ? st.n / 2 : st.n;
  if (tfo.dtype != tin.dtype) return fail(MK_EINVAL, "task '%s': output '%s' has another type than the input", lt.name.c_str(), tfo.name.c_str());
  if (tfo.ndims != 2 || tfo.dims[1] < n_out) return fail(MK_EINVAL, "task '%s': output '%s' has %lld columns, need %d", lt.name.c_str(), tfo.name.c_str(), (long long)tfo.dims[1], n_out);
  if (tin.dims[0] < g->cfg.max_num_batched_tokens || tfo.dims[0] < g->cfg.max_num_batched_tokens)
    return fail(MK_EINVAL, "task '%s': activations need at least max_num_batched_tokens=%d rows", lt.name.c_str(), g->cfg.max_num_batched_tokens);
  st.in = tin.ptr;
  st.ld_in = (int)tin.strides[0];
  st.out = tfo.ptr;
  st.ld_out = (int)tfo.strides[0];
  if (res) {
    const Tensor &tr = g->tensors[res_id];
    if (tr.ndims != 2 || tr.dims[1] < n_out || tr.dtype != MK_DT_BF16) return fail(MK_EINVAL, "task '%s': bad residual '%s'", lt.name.c_str(), tr.name.c_str());
    st.flags |= MK_F_RES;
    st.res = tr.ptr;
    st.ld_res = (int)tr.strides[0];
  }
  if (norm) {
    const Tensor &nx = g->tensors[norm->ops[0]];
    const Tensor &nw = g->tensors[norm->ops[1]];
    const Tensor &no = g->tensors[norm->ops[2]];
    if (nx.ndims != 2 || nx.dims[1] != st.k || nw.elems() != (size_t)st.k || nw.dtype != MK_DT_BF16)
      return fail(MK_EINVAL, "task '%s': norm shapes do not match k=%d", norm->name.c_str(), st.k);
    MkStage ns;
    memset(&ns, 0, sizeof(ns));
    ns.op = MK_OP_NORM;
    ns.flags = MK_F_ONLY_MULTI;
    ns.k = st.k;
    ns.eps = g->cfg.rms_eps;
    ns.in = nx.ptr;
    ns.ld_in = (int)nx.strides[0];
    ns.norm_w = nw.ptr;
    ns.out = no.ptr;
    ns.ld_out = (int)no.strides[0];
    if (!g->stages.empty()) {
      // a plain or residual linear whose whole output this norm reads may leave its split-K sum to the norm stage
      MkStage &pl = g->stages.back();
      const bool rows_ok = (ns.k & 15) == 0 && ns.k / 8 <= 6 * MK_THREADS && (ns.ld_in & 7) == 0 && (ns.ld_out & 7) == 0 && ((uintptr_t)ns.in & 15) == 0;
      const bool res_ok = !(pl.flags & MK_F_RES) || ((pl.ld_res & 7) == 0 && ((uintptr_t)pl.res & 15) == 0);
      if (pl.op == MK_OP_LINEAR && !(pl.flags & MK_F_SILU) && pl.out == ns.in && pl.ld_out == ns.ld_in && pl.n == ns.k && rows_ok && res_ok)
        pl.flags |= MK_F_DEFER_SUM;
    }
    g->stages.push_back(ns);
    g->stage_desc.push_back(fmt("NORM[multi-token only] %s -> %s k=%d", nx.name.c_str(), no.name.c_str(), st.k));
    st.flags |= MK_F_NORM;
    st.in = nx.ptr;
    st.ld_in = (int)nx.strides[0];
    st.norm_w = nw.ptr;
    st.norm_out = no.ptr;
    st.ld_norm = (int)no.strides[0];
  }
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("LINEAR%s%s%s%s %s x %s -> %s n=%d k=%d segs=%d", f32 ? "_F32" : "", (st.flags & MK_F_NORM) ? "+norm" : "", (st.flags & MK_F_RES) ? "+res" : "",
                              (st.flags & MK_F_GELU) ? "+gelu" : (st.flags & MK_F_SILU) ? "+silu" : sq ? "+relu2" : "", tin.name.c_str(), g->tensors[w_id].name.c_str(), tfo.name.c_str(), st.n, st.k,
                              st.w.nseg));
  g->weight_bytes += (int64_t)st.n * st.k * (int64_t)dtype_size(tin.dtype);
  g->stage_weight.resize(g->stages.size(), -1);
  g->stage_weight.back() = w_id;
  g->last_linear_task = (int)i;
  g->last_linear_stage = (int)g->stages.size() - 1;
  i += act || sq ? 2 : consumed_linear;
  return MK_OK;
}

// silu_mul_linear_with_residual [input [tokens, 2I], weight [H, I], residual, output]: out = silu_mul(input) W^T + residual.
// Which columns of `input` are gate and which are up:
//   * `input` was produced by the linear stage right before it through a shuffled [gate ; up] weight view: the view says so;
//   * params[0] > 0 (the builder that interleaved a physical weight passes its group size): groups of
//     [gate x params[0] ; up x params[0]];
//   * otherwise [gate | up] halves, the layout the reference task kernel reads (tasks/mi300/silu_mul_linear_mi300.cuh:40-42,
//     tasks/ampere/silu_mul_linear.cuh:78-80).
// When the producer is that linear stage and no later task reads `input`, the activation moves into the producer's
// epilogue (single rounding, like the fused gate/up task) writing a library-owned [tokens, I] tensor and the gate/up tensor
// itself is no longer written.  Otherwise a standalone activation stage reads `input`.
int lower_silu_mul_linear(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 4) return fail(MK_EINVAL, "silu_mul_linear_with_residual expects 4 operands");
  const Tensor &x = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &r = g->tensors[t.ops[2]], &o = g->tensors[t.ops[3]];
  const int B = g->cfg.max_num_batched_tokens;
  if (x.ndims != 2 || w.ndims != 2 || r.ndims != 2 || o.ndims != 2 || x.dtype != MK_DT_BF16 || o.dtype != MK_DT_BF16 || r.dtype != MK_DT_BF16)
    return fail(MK_EINVAL, "silu_mul_linear_with_residual: operands must be 2-D bf16");
  const int I = (int)w.dims[1], H = (int)w.dims[0];
  if (x.dims[1] != 2 * (int64_t)I || o.dims[1] < H || r.dims[1] < H || x.dims[0] < B || o.dims[0] < B || r.dims[0] < B)
    return fail(MK_EINVAL, "silu_mul_linear_with_residual: input must be [tokens, 2*%d], residual/output [tokens, >=%d]", I, H);
  if (I % 8 || (B > 1 && I % 32)) return fail(MK_EINVAL, "silu_mul_linear_with_residual: intermediate size %d must be a multiple of 8 (32 when batching)", I);
  void *mid = nullptr;
  int rc = dev_alloc(g, &mid, (size_t)B * I * 2);
  if (rc) return rc;
  const bool have_producer = g->last_linear_stage >= 0 && g->last_linear_stage == (int)g->stages.size() - 1;
  MkStage *prev = have_producer ? &g->stages.back() : nullptr;
  if (prev && !(prev->op == MK_OP_LINEAR && prev->out == x.ptr && !(prev->flags & (MK_F_SILU | MK_F_RES)) && prev->n == 2 * I)) prev = nullptr;
  int half = I;
  const char *how = "[gate | up] halves";
  if (prev && prev->w.nseg == 2 && prev->w.seg_rows[0] == prev->w.seg_rows[1]) {
    half = prev->w.seg_rows[0];
    how = "groups of the producer's shuffled weight view";
  } else if (!t.params.empty() && t.params[0] > 0) {
    half = t.params[0];
    how = "groups given by the caller";
  }
  if (half <= 0 || I % half) return fail(MK_EINVAL, "silu_mul_linear_with_residual: gate/up groups of %d rows do not divide the intermediate size %d", half, I);
  // folding stops the gate/up tensor from being written: no later task may read it before some task writes it again
  // (drivers reuse one gate/up buffer for every layer)
  bool read_later = false;
  for (size_t j = i + 1; j < g->ltasks.size() && !read_later; j++) {
    const Task &lt = g->ltasks[j];
    const size_t n_in = lt.ops.size() - (size_t)num_outputs(lt);
    bool rewritten = false;
    for (size_t a = 0; a < lt.ops.size(); a++) {
      if (lt.ops[a] != t.ops[0]) continue;
      if (a < n_in) read_later = true;
      else rewritten = true;
    }
    if (rewritten) break;
  }
  if (prev && !read_later) {
    prev->flags |= MK_F_SILU;
    prev->silu_half = half;
    prev->out = mid;
    prev->ld_out = I;
    g->stage_desc.back() += fmt(" [+silu half=%d (%s) folded in from silu_mul_linear_with_residual; output is library-owned]", half, how);
  } else {
    MkStage a;
    memset(&a, 0, sizeof(a));
    a.op = MK_OP_SILU_MUL;
    a.n = I;
    a.silu_half = half;
    a.groups = I / half;
    a.in = x.ptr;
    a.ld_in = (int)x.strides[0];
    a.out = mid;
    a.ld_out = I;
    g->stages.push_back(a);
    g->stage_desc.push_back(fmt("SILU_MUL %s -> (library) n=%d half=%d (%s)", x.name.c_str(), I, half, how));
  }
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_LINEAR;
  st.flags = MK_F_RES;
  st.k = I;
  int64_t rows;
  int halfw;
  rc = resolve_weight(g, t.ops[1], I, &st.w, &rows, &halfw);
  if (rc) return rc;
  st.n = (int)rows;
  st.eps = g->cfg.rms_eps;
  st.in = mid;
  st.ld_in = I;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  st.res = r.ptr;
  st.ld_res = (int)r.strides[0];
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("LINEAR+res silu_mul(%s) x %s -> %s n=%d k=%d", x.name.c_str(), w.name.c_str(), o.name.c_str(), st.n, st.k));
  g->weight_bytes += (int64_t)st.n * st.k * 2;
  g->stage_weight.resize(g->stages.size(), -1);
  g->stage_weight.back() = t.ops[1];
  i++;
  return MK_OK;
}

// A merge task that closes a split-KV attention task: [lse, chunked output, final output].  Returns the final
// output's tensor id when task `j` is such a merge over the attention's chunked output, -1 otherwise.
int merge_output_of(mk_graph *g, size_t j, const char *merge_name, int chunked_out_id) {
  if (j >= g->ltasks.size()) return -1;
  const Task &m = g->ltasks[j];
  if (m.name != merge_name || m.ops.size() != 3 || m.ops[1] != chunked_out_id) return -1;
  return m.ops[2];
}

// Every attention flavour of the API becomes ONE stage (q/k-norm, RoPE, KV append, attention over a KV split the stage
// chooses itself, merge): the fused tasks directly, kv_cache_update + attention as a pair, and any of them built with
// num_kv_chunks > 1 together with the merge task that must follow (the stage writes the merge's output; the chunked
// accumulator and the log-sum-exp tensor of the reference's two-task form are never touched).
int lower_attention(mk_graph *g, size_t &i) {
  const Task &t0 = g->ltasks[i];
  int in_id, kc_id, vc_id, qn_id, kn_id, cos_id, sin_id, out_id, qws_id = -1, nq = 0, chunks = 1;
  size_t consumed = 1;
  const char *merge = nullptr;
  if (t0.name == "gang_attn_split_kv_mi300") {
    if (t0.ops.size() != 10 || t0.params.size() < 10) return fail(MK_EINVAL, "gang_attn_split_kv_mi300 expects 10 operands / 10 params");
    in_id = t0.ops[0]; kc_id = t0.ops[1]; vc_id = t0.ops[2]; qn_id = t0.ops[3]; kn_id = t0.ops[4]; cos_id = t0.ops[5]; sin_id = t0.ops[6];
    out_id = t0.ops[8]; qws_id = t0.ops[9];
    nq = t0.params[0];
    chunks = t0.params[6];
    merge = "gang_attn_merge_mi300";
  } else if (t0.name == "paged_attention" || t0.name == "paged_attention_split_kv_mi300" || t0.name == "attention" || t0.name == "single_batch_extend_attention") {
    // "attention" (python/mirage/mpk/persistent_kernel.py:587-650) is the form with one contiguous cache row range per
    // request, [requests, seq_len, kv heads, head_dim]: a paged cache whose pages are max_seq_length long
    const bool split = t0.name == "paged_attention_split_kv_mi300";
    // ("single_batch_extend_attention", persistent_kernel.py:653-730: the same cache form for the rows of a speculating
    // request -- its newest token and the guesses behind it; params 4, 5 = number of guesses, output stride)
    const size_t need_params = t0.name == "attention" ? 4u : (split ? 7u : 6u);
    if (t0.ops.size() != (split ? 9u : 8u) || t0.params.size() < need_params) return fail(MK_EINVAL, "%s: wrong number of operands / params", t0.name.c_str());
    in_id = t0.ops[0]; kc_id = t0.ops[1]; vc_id = t0.ops[2]; qn_id = t0.ops[3]; kn_id = t0.ops[4]; cos_id = t0.ops[5]; sin_id = t0.ops[6];
    out_id = t0.ops.back();
    nq = t0.params[0];
    if (split) {
      chunks = 2;  // the chunked [tokens, chunks * heads * head_dim, kv heads] output always needs the merge task
      merge = "paged_attention_split_kv_merge_mi300";
    }
  } else if (t0.name == "kv_cache_update_mi300") {
    if (t0.ops.size() != 8 || t0.params.size() < 7) return fail(MK_EINVAL, "kv_cache_update_mi300 expects 8 operands / 7 params");
    if (i + 1 >= g->ltasks.size() || g->ltasks[i + 1].name != "paged_attention_ck_fmha_split_kv_mi300")
      return fail(MK_EUNSUPPORTED, "kv_cache_update_mi300 must be followed by paged_attention_ck_fmha_split_kv_mi300");
    const Task &t1 = g->ltasks[i + 1];
    if (t1.ops.size() != 5 || t1.params.size() < 9) return fail(MK_EINVAL, "paged_attention_ck_fmha_split_kv_mi300 expects 5 operands / 9 params");
    in_id = t0.ops[0]; kc_id = t0.ops[1]; vc_id = t0.ops[2]; qn_id = t0.ops[3]; kn_id = t0.ops[4]; cos_id = t0.ops[5]; sin_id = t0.ops[6];
    qws_id = t0.ops[7];
    if (t1.ops[0] != qws_id || t1.ops[1] != kc_id || t1.ops[2] != vc_id) return fail(MK_EINVAL, "attention does not consume the q workspace / caches of the preceding kv_cache_update");
    out_id = t1.ops[3];
    nq = t0.params[0];
    chunks = t1.params[5];
    merge = "paged_attention_ck_fmha_merge_mi300";
    consumed = 2;
  } else {
    return fail(MK_EUNSUPPORTED, "attention task '%s' is not supported", t0.name.c_str());
  }
  if (chunks < 1) return fail(MK_EINVAL, "%s: num_kv_chunks=%d", t0.name.c_str(), chunks);
  if (chunks > 1) {
    const int fin = merge_output_of(g, i + consumed, merge, out_id);
    if (fin < 0) return fail(MK_EUNSUPPORTED, "%s with num_kv_chunks=%d must be followed by %s over its chunked output", t0.name.c_str(), chunks, merge);
    out_id = fin;
    consumed++;
  }
  const Tensor &tin = g->tensors[in_id], &kc = g->tensors[kc_id], &vc = g->tensors[vc_id], &to = g->tensors[out_id];
  if (kc.ndims != 4 || vc.ndims != 4) return fail(MK_EINVAL, "k/v cache must be 4-D [pages, page_size, kv_heads, head_dim]");
  const int nkv = (int)kc.dims[2], D = (int)kc.dims[3];
  if (D != 128) return fail(MK_EUNSUPPORTED, "head_dim %d: only 128 is supported", D);
  if (kc.dims[0] < g->cfg.max_num_pages || vc.dims[0] < g->cfg.max_num_pages)
    return fail(MK_EINVAL, "k/v cache holds %lld / %lld pages, fewer than max_num_pages=%d", (long long)kc.dims[0], (long long)vc.dims[0], g->cfg.max_num_pages);
  for (int d = 1; d < 4; d++)
    if (kc.dims[d] != vc.dims[d]) return fail(MK_EINVAL, "k and v cache shapes differ");
  if (kc.dtype != MK_DT_BF16 || vc.dtype != MK_DT_BF16) return fail(MK_EINVAL, "k/v cache must be bf16");
  if (kc.dims[1] != g->cfg.page_size) return fail(MK_EINVAL, "k cache page size %lld != configured %d", (long long)kc.dims[1], g->cfg.page_size);
  if (nkv <= 0 || nq % nkv) return fail(MK_EINVAL, "q heads %d not a multiple of kv heads %d", nq, nkv);
  const int qpk = nq / nkv;
  if (qpk != 4 && qpk != 8) return fail(MK_EUNSUPPORTED, "q heads per kv head = %d: supported 4 and 8", qpk);
  if (tin.ndims != 2 || tin.dims[1] != (int64_t)(nq + 2 * nkv) * D) return fail(MK_EINVAL, "attention input must be [tokens, (q+2kv)*head_dim]");
  if (to.ndims != 2 || to.dims[1] < (int64_t)nq * D) return fail(MK_EINVAL, "attention output must be [tokens, q_heads*head_dim]");
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_ATTN;
  st.eps = g->cfg.rms_eps;
  st.in = tin.ptr;
  st.ld_in = (int)tin.strides[0];
  st.out = to.ptr;
  st.ld_out = (int)to.strides[0];
  st.k_cache = kc.ptr;
  st.v_cache = vc.ptr;
  st.num_q_heads = nq;
  st.num_kv_heads = nkv;
  st.head_dim = D;
  st.sm_scale_log2 = (float)(1.4426950408889634 / sqrt((double)D));
  if (qn_id >= 0 && kn_id >= 0) {
    st.flags |= MK_F_QK_NORM;
    st.q_norm_w = g->tensors[qn_id].ptr;
    st.k_norm_w = g->tensors[kn_id].ptr;
    if (g->tensors[qn_id].elems() != (size_t)D || g->tensors[kn_id].elems() != (size_t)D) return fail(MK_EINVAL, "q/k norm weights must have head_dim elements");
  }
  if (cos_id >= 0 && sin_id >= 0) {
    const Tensor &c = g->tensors[cos_id];
    if (c.ndims != 2 || c.dims[1] < D / 2 || c.dims[0] < g->cfg.max_seq_length) return fail(MK_EINVAL, "cos/sin tables must be [>=max_seq_length, >=head_dim/2]");
    st.flags |= MK_F_ROPE;
    st.cos_tab = c.ptr;
    st.sin_tab = g->tensors[sin_id].ptr;
    st.ld_cos = (int)c.strides[0];
  }
  if (qws_id >= 0) {
    st.q_ws = g->tensors[qws_id].ptr;
    st.ld_qws = (int)g->tensors[qws_id].strides[0];
  }
  if (!g->stages.empty()) {
    // a plain linear whose whole output is this stage's q/k/v rows may leave its split-K sum to this stage's row fetch
    MkStage &pl = g->stages.back();
    if (pl.op == MK_OP_LINEAR && !(pl.flags & (MK_F_SILU | MK_F_RES)) && pl.out == st.in && pl.ld_out == st.ld_in && pl.n == (nq + 2 * nkv) * D)
      pl.flags |= MK_F_DEFER_SUM;
  }
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("ATTN %s -> %s q=%d kv=%d d=%d norm=%d rope=%d", tin.name.c_str(), to.name.c_str(), nq, nkv, D, !!(st.flags & MK_F_QK_NORM),
                              !!(st.flags & MK_F_ROPE)));
  i += consumed;
  return MK_OK;
}


// ---- flex tasks (mk_flex.hip): sizes and constants are data --------------------------------------------------------
// embedding_scaled [ids, table, residual rows (fp32), rows] params [source, scale bits]; with one more operand behind the table, [positions,
// table columns]: its row at the token's position is added (behind the last row: the last one).
int lower_embedding_scaled(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  const bool ext = t.ops.size() == 5;
  if ((!ext && t.ops.size() != 4) || t.params.size() != 2) return fail(MK_EINVAL, "embedding_scaled expects 4 or 5 operands / 2 params");
  const Tensor &ids = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &r = g->tensors[t.ops[2 + ext]], &o = g->tensors[t.ops[3 + ext]];
  const int B = g->cfg.max_num_batched_tokens;
  if (ids.dtype != MK_DT_I64 || (int64_t)ids.elems() < B) return fail(MK_EINVAL, "embedding_scaled: ids must be int64, one per token row");
  if (w.ndims != 2 || o.ndims != 2 || r.ndims != 2 || o.dims[1] < w.dims[1] || r.dims[1] < w.dims[1] || o.dims[0] < B || r.dims[0] < B || w.dtype != o.dtype || r.dtype != MK_DT_F32 ||
      w.kind == T_SHUFFLED || (o.strides[0] & 3) || (r.strides[0] & 3))
    return fail(MK_EINVAL, "embedding_scaled shapes mismatch");
  int rc = set_flex(g, o.dtype, "embedding_scaled");
  if (rc) return rc;
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_FX_EMBED;
  st.k = (int)w.dims[1];
  st.in = ids.ptr;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  st.out2 = r.ptr == o.ptr ? nullptr : r.ptr;
  st.ld_out2 = (int)r.strides[0];
  st.alpha = bits_f32(t.params[1]);
  st.w.nseg = 1;
  st.w.seg[0] = w.ptr;
  if (t.params[0] == 0) st.flags |= MK_F_EMBED_FROM_TOKENS;
  if (ext) {
    const Tensor &pos = g->tensors[t.ops[2]];
    if (pos.ndims != 2 || pos.dims[0] < 1 || pos.dims[1] != w.dims[1] || pos.strides[0] != w.dims[1] || pos.dtype != w.dtype) return fail(MK_EINVAL, "embedding_scaled: position vectors are [positions, %d] of the table's type", st.k);
    st.pos_tab = pos.ptr;
    st.pos_rows = (int)pos.dims[0];
    g->mix = g->hyb = g->dual = true;
  }
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("FX_EMBED %s[%s] * %g%s -> %s, %s k=%d", w.name.c_str(), ids.name.c_str(), st.alpha, ext ? " + position" : "", r.name.c_str(), o.name.c_str(), st.k));
  i++;
  return MK_OK;
}

// residual_rmsnorm [y (optional), residual (fp32), weight (fp32), new residual (fp32), rows] params [width, alpha bits, eps
// bits, weight offset bits]: v = alpha * residual + y, both outputs = v / rms(v) * (offset + weight).  A bf16 linear that
// reads the rows next forms them itself when an iteration has one token; a linear that wrote y may leave its K-slice sum.
int lower_residual_rmsnorm(mk_graph *g, size_t &i) {
  const Task t = g->ltasks[i];
  if (t.ops.size() != 5 || t.params.size() != 4) return fail(MK_EINVAL, "residual_rmsnorm expects 5 operands / 4 params");
  const Tensor *y = t.ops[0] >= 0 ? &g->tensors[t.ops[0]] : nullptr;
  const Tensor x = g->tensors[t.ops[1]], w = g->tensors[t.ops[2]], xo = g->tensors[t.ops[3]], o = g->tensors[t.ops[4]];
  const int B = g->cfg.max_num_batched_tokens, width = t.params[0];
  const int64_t n = o.dims[1];
  int rc = set_flex(g, o.dtype, "residual_rmsnorm");
  if (rc) return rc;
  if (o.ndims != 2 || x.ndims != 2 || xo.ndims != 2 || n % 4 || width < 1 || width > n || x.dims[1] != n || xo.dims[1] != n || (int64_t)w.elems() != n ||
      (y && (y->ndims != 2 || y->dims[1] != n || y->dtype != o.dtype || y->dims[0] < B)) || o.dims[0] < B || x.dims[0] < B || xo.dims[0] < B)
    return fail(MK_EINVAL, "residual_rmsnorm: every row tensor is [tokens, %lld] (a multiple of 4), the weight has as many entries, width=%d of them real", (long long)n, width);
  if (x.dtype != MK_DT_F32 || xo.dtype != MK_DT_F32 || w.dtype != MK_DT_F32) return fail(MK_EINVAL, "residual_rmsnorm: residual rows and norm weight are fp32");
  if (n > 12 * 4 * MK_THREADS) return fail(MK_EUNSUPPORTED, "residual_rmsnorm: rows of %lld values (most %d)", (long long)n, 12 * 4 * MK_THREADS);
  if (x.ptr == xo.ptr && xo.ptr != o.ptr) return fail(MK_EINVAL, "residual_rmsnorm: the new residual rows must not overwrite the old ones (other workgroups may still read them)");
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_FX_ADDNORM;
  st.n = (int)n;
  st.k = width;
  st.alpha = bits_f32(t.params[1]);
  st.eps = bits_f32(t.params[2]);
  st.w_offset = bits_f32(t.params[3]);
  st.in = y ? y->ptr : nullptr;
  st.ld_in = y ? (int)y->strides[0] : 0;
  st.res = x.ptr;
  st.ld_res = (int)x.strides[0];
  st.norm_w = w.ptr;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  st.out2 = xo.ptr == o.ptr ? nullptr : xo.ptr;
  st.ld_out2 = (int)xo.strides[0];
  if ((st.ld_in | st.ld_res | st.ld_out | st.ld_out2) & 3) return fail(MK_EINVAL, "residual_rmsnorm: row strides must be multiples of 4");
  if (!g->stages.empty()) {
    MkStage &pl = g->stages.back();
    if (pl.op == MK_OP_LINEAR && !(pl.flags & (MK_F_SILU | MK_F_RES)) && y && pl.out == st.in && pl.ld_out == st.ld_in && pl.n == st.n && width == n)
      pl.flags |= MK_F_DEFER_SUM;
    if (pl.out != st.res && pl.out2 != st.res && pl.norm_out != st.res) st.flags |= MK_F_RES_EARLY;
  }
  bool res, silu;
  int extra;
  const bool fuse = g->flex == FLEX_BF16 && i + 1 < g->ltasks.size() && linear_kind(g->ltasks[i + 1].name, &res, &silu, &extra) && !res && g->ltasks[i + 1].ops[0] == t.ops[4];
  if (fuse) st.flags |= MK_F_ONLY_MULTI;
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("FX_ADDNORM%s %g * %s + %s -> %s, %s k=%d", fuse ? "[multi-token only]" : "", st.alpha, x.name.c_str(), y ? y->name.c_str() : "0", xo.name.c_str(), o.name.c_str(), width));
  i++;
  if (!fuse) return MK_OK;
  rc = lower_linear(g, i);
  if (rc) return rc;
  MkStage &l = g->stages.back();
  l.flags |= MK_F_NORM | MK_F_ADDNORM | (st.flags & MK_F_RES_EARLY);
  l.y_in = st.in;
  l.ld_y = st.ld_in;
  l.res = st.res;
  l.ld_res = st.ld_res;
  l.norm_w = st.norm_w;
  l.norm_out = st.out;
  l.ld_norm = st.ld_out;
  l.out2 = st.out2;
  l.ld_out2 = st.ld_out2;
  l.alpha = st.alpha;
  l.w_offset = st.w_offset;
  l.norm_eps = st.eps;
  l.k_real = width;
  return MK_OK;
}

// flex_attention [qkv rows, k cache, v cache, cos (optional), sin (optional), sink (optional), q workspace, output]
// params [q heads, kv heads, head dim, value dim, rotated dims, unit norm 0/1, eps bits, scale bits, softcap bits].  The
// qkv rows are all query heads, then all key heads, then all value heads; caches are [pages, page_size, kv heads, padded
// dim] with a layout of the library's own inside a page.  With three more params [window, kept first positions, values from
// keys 0/1] and one more operand behind the sink, fp32 [input columns] added to the rows: a position sees the `window` newest
// ones and the kept first ones; the value heads are the key heads before rotation (the rows hold no others).  With one more param and
// three more operands behind those [q row weights, k row weights, score factors; all optional]: a position sees only its own chunk
// (param, 0: none) of positions; all query heads of a row are divided by their common root mean square and multiplied by a
// weight per column, all key heads likewise; scores are multiplied by a factor per head.
int lower_flex_attention(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  const bool ext2 = t.ops.size() == 12 && t.params.size() == 13, ext = ext2 || (t.ops.size() == 9 && t.params.size() == 12);
  if (!ext && (t.ops.size() != 8 || t.params.size() != 9)) return fail(MK_EINVAL, "flex_attention expects 8 operands / 9 params, or 9 / 12, or 12 / 13");
  const Tensor &in = g->tensors[t.ops[0]], &kc = g->tensors[t.ops[1]], &vc = g->tensors[t.ops[2]], &qw = g->tensors[t.ops[t.ops.size() - 2]], &o = g->tensors[t.ops.back()];
  const int window = ext ? t.params[9] : 0, keep = ext ? t.params[10] : 0, own_v = !(ext && t.params[11]);
  const int B = g->cfg.max_num_batched_tokens, ps = g->cfg.page_size;
  const int H = t.params[0], G = t.params[1], D = t.params[2], DV = t.params[3], rot = t.params[4];
  int rc = set_flex(g, in.dtype, "flex_attention");
  if (rc) return rc;
  const bool f32 = in.dtype == MK_DT_F32;
  const int es = f32 ? 4 : 2, KW = f32 ? 16 : 32, TP = f32 ? 16 : 32;
  if (H < 1 || G < 1 || H % G || D < 1 || DV < 1 || rot < 0 || rot > D || rot % 2) return fail(MK_EINVAL, "flex_attention: heads %d / %d, dims %d / %d, rotated %d", H, G, D, DV, rot);
  if (D > MK_FX_MAX_HEAD_DIM || DV > MK_FX_MAX_HEAD_DIM) return fail(MK_EUNSUPPORTED, "flex_attention: head dims %d / %d (most %d)", D, DV, MK_FX_MAX_HEAD_DIM);
  const int dk = (D + KW - 1) / KW * KW, dv = (DV + 15) / 16 * 16;
  const int64_t cols = (int64_t)H * D + (int64_t)G * (D + own_v * DV);
  if (window < 0 || keep < 0 || (!own_v && D != DV)) return fail(MK_EINVAL, "flex_attention: window %d, %d kept positions, key / value size %d / %d", window, keep, D, DV);
  if (ext && t.ops[6] >= 0 && !vector_ok(g->tensors[t.ops[6]], cols)) return fail(MK_EINVAL, "flex_attention: the bias holds one fp32 value per input column");
  if (in.ndims != 2 || in.dims[0] < B || in.dims[1] < (int64_t)H * D + (int64_t)G * (D + own_v * DV)) return fail(MK_EINVAL, "flex_attention: input must be [tokens, >= (q + kv) * dim + kv * value dim]");
  if (o.ndims != 2 || o.dims[0] < B || o.dims[1] < (int64_t)H * DV || o.dtype != in.dtype) return fail(MK_EINVAL, "flex_attention: output must be [tokens, >= q heads * value dim] of the input's type");
  if (qw.ndims != 2 || qw.dims[0] < B || qw.dims[1] < (int64_t)H * dk || qw.dtype != in.dtype || (qw.strides[0] * es) % 16) return fail(MK_EINVAL, "flex_attention: q workspace must be [tokens, >= q heads * %d]", dk);
  if (kc.ndims != 4 || vc.ndims != 4 || kc.dtype != in.dtype || vc.dtype != in.dtype || kc.dims[0] < g->cfg.max_num_pages || vc.dims[0] < g->cfg.max_num_pages || kc.dims[1] != ps ||
      vc.dims[1] != ps || kc.dims[2] != G || vc.dims[2] != G || kc.dims[3] != dk || vc.dims[3] != dv)
    return fail(MK_EINVAL, "flex_attention: caches must be [>= %d pages, %d, %d, %d] and [.., %d], of the input's type", g->cfg.max_num_pages, ps, G, dk, dv);
  if (ps % TP) return fail(MK_EINVAL, "flex_attention: page_size %d must be a multiple of %d", ps, TP);
  if ((int64_t)kc.elems() / 8 > 0x7fffffffll * 16) return fail(MK_EUNSUPPORTED, "flex_attention: cache too large");
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_FX_ATTN;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  st.k_cache = kc.ptr;
  st.v_cache = vc.ptr;
  st.q_ws = qw.ptr;
  st.ld_qws = (int)qw.strides[0];
  st.num_q_heads = H;
  st.num_kv_heads = G;
  st.head_dim = D;
  st.v_dim = DV;
  st.v_col = own_v ? (H + G) * D : H * D;
  st.window = window;
  st.keep_first = window ? keep : 0;
  st.in_bias = ext && t.ops[6] >= 0 ? (const float *)g->tensors[t.ops[6]].ptr : nullptr;
  if (ext) g->mix = g->hyb = true;
  if (ext2) {
    const int qn = t.ops[7], kn = t.ops[8], tp = t.ops[9];
    if (t.params[12] < 0 || (qn >= 0) != (kn >= 0) || (qn >= 0 && (t.params[5] || rot || st.in_bias || !vector_ok(g->tensors[qn], (int64_t)H * D) || !vector_ok(g->tensors[kn], (int64_t)G * D))) ||
        (tp >= 0 && !vector_ok(g->tensors[tp], H)))
      return fail(MK_EINVAL, "flex_attention: chunks of %d; row norms need fp32 weights for all query and all key columns, and no rotation, bias or unit norm beside them; a score factor per head", t.params[12]);
    g->dual = true;
    st.chunk = t.params[12];
    if (qn >= 0) {
      st.flags |= MK_F_ROW_NORM;
      st.q_norm_w = g->tensors[qn].ptr;
      st.k_norm_w = g->tensors[kn].ptr;
    }
    st.temp = tp >= 0 ? (const float *)g->tensors[tp].ptr : nullptr;
  }
  st.rot_dims = rot;
  st.eps = bits_f32(t.params[6]);
  st.sm_scale = bits_f32(t.params[7]);
  st.softcap = bits_f32(t.params[8]);
  if (t.params[5]) st.flags |= MK_F_QK_NORM;
  if (rot > 0) {
    if (t.ops[3] < 0 || t.ops[4] < 0) return fail(MK_EINVAL, "flex_attention: rotated dims without cos / sin tables");
    const Tensor &c = g->tensors[t.ops[3]], &s = g->tensors[t.ops[4]];
    if (c.dtype != MK_DT_F32 || s.dtype != MK_DT_F32 || c.ndims != 2 || s.ndims != 2 || c.dims[1] != rot / 2 || s.dims[1] != rot / 2 || c.dims[0] < g->cfg.max_seq_length ||
        s.dims[0] < g->cfg.max_seq_length || c.strides[0] != s.strides[0])
      return fail(MK_EINVAL, "flex_attention: cos / sin tables must be fp32 [>= max_seq_length, rotated dims / 2]");
    st.flags |= MK_F_ROPE;
    st.cos_tab = c.ptr;
    st.sin_tab = s.ptr;
    st.ld_cos = (int)c.strides[0];
  }
  if (t.ops[5] >= 0) {
    const Tensor &s = g->tensors[t.ops[5]];
    if (s.dtype != MK_DT_F32 || (int64_t)s.elems() != H) return fail(MK_EINVAL, "flex_attention: the sink holds one fp32 value per query head");
    st.sink = s.ptr;
  }
  // instantiation: 16-byte key operand rows and 16-wide value blocks a tile load holds (mk_flex.hip: stage_fx_attn)
  st.k_tiles = f32 ? 8 : (dk <= 64 && dv <= 64 ? 2 : 4);
  st.v_tiles = f32 ? 8 : (dv <= 64 ? 4 : 8);
  const int nkc = dk / KW, nkg = (nkc + st.k_tiles - 1) / st.k_tiles, nvs = (dv / 16 + st.v_tiles - 1) / st.v_tiles;
  const int64_t pages = ((int64_t)g->cfg.max_seq_length + ps - 1) / ps;
  const int64_t lds = (int64_t)nkg * st.k_tiles * 1024 + (int64_t)(dk + dv) * es + 16 + 4 * 16 * (st.v_tiles * 16 + 4) * 4 + (128 + 96 + 2 * MK_ATTN_MAX_CHUNKS * 16 + 4) * 4 + pages * 4;
  if (lds > MK_LDS_BYTES) return fail(MK_EUNSUPPORTED, "flex_attention: needs %lld bytes of LDS (head dim %d, %lld pages per request)", (long long)lds, D, (long long)pages);
  const size_t items = (size_t)B * ((H / G + 15) / 16) * G * nvs;
  g->flex_items = std::max(g->flex_items, items);
  g->flex_part = std::max(g->flex_part, (size_t)g->G * 16 * (st.v_tiles * 16 + 32));
  if (!g->stages.empty()) {
    MkStage &pl = g->stages.back();  // the q/k/v linear may leave its K-slice sum to this stage's row fetch
    if (pl.op == MK_OP_LINEAR && !(pl.flags & (MK_F_SILU | MK_F_RES)) && pl.out == st.in && pl.ld_out == st.ld_in && pl.n >= cols && !(st.flags & MK_F_ROW_NORM)) pl.flags |= MK_F_DEFER_SUM;
  }
  if (B > 1) {
    MkStage sp = st;
    sp.op = MK_OP_FX_PREP;
    g->stages.push_back(sp);
    g->stage_desc.push_back(fmt("FX_PREP[portions] %s", in.name.c_str()));
  }
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("FX_ATTN %s -> %s q=%d kv=%d d=%d dv=%d rot=%d norm=%d softcap=%g sink=%d window=%d+%d bias=%d chunk=%d rownorm=%d", in.name.c_str(), o.name.c_str(), H, G, D, DV, rot, t.params[5], st.softcap, t.ops[5] >= 0, st.window, st.keep_first, st.in_bias != nullptr, st.chunk, !!(st.flags & MK_F_ROW_NORM)));
  i++;
  return MK_OK;
}

// ---- mix tasks (mk_mix.hip) --------------------------------------------------------------------------------------------

int set_mix(mk_graph *g, int dtype, const char *task) {
  g->mix = true;
  return set_flex(g, dtype, task);
}

// residual_prenorm [y (optional), y weight (fp32, optional), residual (fp32), weight (fp32, optional), new residual (fp32), rows]
// params [width, groups, alpha bits, eps bits, y eps bits]: v = residual + alpha * y (with a y weight: of the RMS-normalised
// y); new residual = v, rows = the RMS norm of v in `groups` equal parts times weight (no weight: v).  A bf16 linear that
// reads the rows next forms them itself when an iteration has one token.
// With two more operands behind the y weight (fp32 [columns] added to y, optional; fp32 [tokens, >= slots] weights, optional) and
// two more params [slots, columns per slot]: y is the weighted sum of `slots` rows that lie side by side.  With three more operands
// behind those (y factor, y2, y2 factor; factors are fp32 [columns], all optional): v = residual + alpha * y factor * y + y2 factor * y2,
// and the slots belong to y2.  The new residual rows are optional then.  A ring_conv that adds the rows' convolution to them right behind is
// done by this stage when every request brings one token, and the linear may follow that.
int lower_ring_conv(mk_graph *g, size_t &i, MkStage *out, std::string *desc);
int lower_residual_prenorm(mk_graph *g, size_t &i) {
  const Task t = g->ltasks[i];
  const bool ext2 = t.ops.size() == 11 && t.params.size() == 7, ext = ext2 || (t.ops.size() == 8 && t.params.size() == 7);
  const int e2 = ext2 ? 5 : ext ? 2 : 0;
  if (!ext && (t.ops.size() != 6 || t.params.size() != 5)) return fail(MK_EINVAL, "residual_prenorm expects 6 operands / 5 params, or 8 / 7, or 11 / 7");
  auto opt = [&](int k) { return t.ops[k] >= 0 ? &g->tensors[t.ops[k]] : nullptr; };
  const Tensor *y = opt(0), *yw = opt(1), *yb = ext ? opt(2) : nullptr, *sw = ext ? opt(3) : nullptr, *w = opt(3 + e2);
  const Tensor *ys = ext2 ? opt(4) : nullptr, *y2 = ext2 ? opt(5) : nullptr, *y2s = ext2 ? opt(6) : nullptr, *ys_of = sw && y2 ? y2 : y;
  const bool no_xo = t.ops[4 + e2] < 0;
  if (no_xo && (!ext2 || !w)) return fail(MK_EINVAL, "residual_prenorm: the new residual rows are missing");
  const Tensor x = g->tensors[t.ops[2 + e2]], o = g->tensors[t.ops[5 + e2]], xo = no_xo ? x : g->tensors[t.ops[4 + e2]];
  const int slots = sw ? t.params[5] : 0, ld_slot = sw ? t.params[6] : 0;
  const int B = g->cfg.max_num_batched_tokens, width = t.params[0], groups = t.params[1];
  const int64_t n = o.ndims == 2 ? o.dims[1] : 0;
  int rc = set_mix(g, o.dtype, "residual_prenorm");
  if (rc) return rc;
  if (n < 4 || n % 4 || width < 1 || width > n || !rows_ok(o, B, n, o.dtype) || !rows_ok(x, B, n, MK_DT_F32) || !rows_ok(xo, B, n, MK_DT_F32) || x.dims[1] != n || xo.dims[1] != n ||
      (y && (!rows_ok(*y, B, n, o.dtype) || (!(sw && !y2) && y->dims[1] != n))) || (y2 && (!y || !rows_ok(*y2, B, n, o.dtype) || (!sw && y2->dims[1] != n))) || (ys && (!y || !vector_ok(*ys, n))) ||
      (y2s && (!y2 || !vector_ok(*y2s, n))) || (w && !vector_ok(*w, n)) || (yw && (!y || !vector_ok(*yw, n))))
    return fail(MK_EINVAL, "residual_prenorm: every row tensor is [tokens, %lld] (a multiple of 4; residual fp32), weights are fp32 of that size, width=%d of it real", (long long)n, width);
  if (w && (groups < 1 || groups > MK_MX_MAX_GROUPS || width % groups)) return fail(MK_EINVAL, "residual_prenorm: %d parts of a row of %d (at most %d)", groups, width, MK_MX_MAX_GROUPS);
  if ((yb && (!y || !vector_ok(*yb, n))) || (sw && (!y || (yb && !y2) || slots < 1 || slots > MK_MOE_MAX_TOPK + 1 || ld_slot < n || ld_slot % 8 || ys_of->dims[1] < (int64_t)(slots - 1) * ld_slot + n || !rows_ok(*sw, B, slots, MK_DT_F32))))
    return fail(MK_EINVAL, "residual_prenorm: a bias has %lld entries; %d slots of %d columns with fp32 weights of that many columns (and no bias)", (long long)n, slots, ld_slot);
  if (n > 12 * 4 * MK_THREADS) return fail(MK_EUNSUPPORTED, "residual_prenorm: rows of %lld values (most %d)", (long long)n, 12 * 4 * MK_THREADS);
  if (!no_xo && (x.ptr == xo.ptr || (xo.ptr == o.ptr && w))) return fail(MK_EINVAL, "residual_prenorm: the new residual rows must not overwrite the old ones (other workgroups may still read them), nor the rows them");
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_MX_PRENORM;
  st.n = (int)n;
  st.k = width;
  st.norm_groups = w ? groups : 0;
  st.alpha = bits_f32(t.params[2]);
  st.eps = bits_f32(t.params[3]);
  st.norm_eps = bits_f32(t.params[4]);
  st.in = y ? y->ptr : nullptr;
  st.ld_in = y ? (int)y->strides[0] : 0;
  st.y_norm_w = yw ? yw->ptr : nullptr;
  st.in_bias = yb ? (const float *)yb->ptr : nullptr;
  st.slots = slots;
  st.ld_slot = ld_slot;
  st.slot_w = sw ? (const float *)sw->ptr : nullptr;
  st.ld_slot_w = sw ? (int)sw->strides[0] : 0;
  if (yb || sw) g->hyb = true;
  if (ext2) g->hyb = g->dual = true;
  st.y_scale = ys ? (const float *)ys->ptr : nullptr;
  st.y2 = y2 ? y2->ptr : nullptr;
  st.ld_y2 = y2 ? (int)y2->strides[0] : 0;
  st.y2_scale = y2s ? (const float *)y2s->ptr : nullptr;
  st.res = x.ptr;
  st.ld_res = (int)x.strides[0];
  st.norm_w = w ? w->ptr : nullptr;
  st.out = xo.ptr == o.ptr ? nullptr : o.ptr;
  st.ld_out = (int)o.strides[0];
  st.out2 = no_xo ? nullptr : xo.ptr;
  st.ld_out2 = (int)xo.strides[0];
  if (!g->stages.empty()) {
    MkStage &pl = g->stages.back();
    if (!w && !yw && !yb && !sw && !ys && !y2 && y && st.out && pl.op == MK_OP_LINEAR && !(pl.flags & (MK_F_SILU | MK_F_RES)) && pl.out == st.in && (pl.k & 63) == 0) {
      // a plain linear in front adds its single-token result to the stream itself
      pl.flags |= MK_F_JOIN;
      pl.res = st.res;
      pl.ld_res = st.ld_res;
      pl.out2 = st.out2;
      pl.ld_out2 = st.ld_out2;
      pl.norm_out = st.out;
      pl.ld_norm = st.ld_out;
      pl.alpha = st.alpha;
      st.flags |= MK_F_ONLY_MULTI;
    }
    if (pl.out != st.res && pl.out2 != st.res && pl.norm_out != st.res) st.flags |= MK_F_RES_EARLY;
  }
  bool res, silu;
  int extra;
  i++;
  int rows_id = t.ops[5 + e2];
  MkStage conv;
  std::string conv_desc;
  if (w && st.out && i < g->ltasks.size() && g->ltasks[i].name == "ring_conv" && g->ltasks[i].ops.size() == 9 && g->ltasks[i].ops[0] == rows_id && g->ltasks[i].params.size() == 6 &&
      g->ltasks[i].params[0] == 0 && g->ltasks[i].params[2] && !g->ltasks[i].params[1] && g->ltasks[i].ops[2] < 0 && g->ltasks[i].ops[5] < 0) {
    rows_id = g->ltasks[i].ops[7];
    if ((rc = lower_ring_conv(g, i, &conv, &conv_desc))) return rc;
    if (conv.n != n) return fail(MK_EINVAL, "ring_conv: %d channels over rows of %lld", conv.n, (long long)n);
    conv.flags |= MK_F_PORTIONS;
    st.conv_w = conv.conv_w;
    st.taps = conv.taps;
    st.tail = conv.tail;
    st.out3 = conv.out;
    st.ld_out3 = conv.ld_out;
  }
  bool fuse = g->flex == FLEX_BF16 && w && i < g->ltasks.size() && linear_kind(g->ltasks[i].name, &res, &silu, &extra) && !res && g->ltasks[i].ops[0] == rows_id;
  if (fuse && (ys || y2 || st.conv_w)) {  // these forms: a plain linear, one part of the norm, nothing else in front
    const std::string behind = i + 1 < g->ltasks.size() ? g->ltasks[i + 1].name : "";
    fuse = !silu && !yw && !yb && groups == 1 && n % 64 == 0 && behind != "silu_mul" && behind != "gelu_mul" && behind != "silu_mul_linear_with_residual";
  }
  // rows that are only normalised: a stage whose wavefronts share the parts is faster than every workgroup of the linear reading all of them
  if (!y && no_xo) fuse = false;
  if (fuse) st.flags |= MK_F_ONLY_MULTI;
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MX_PRENORM%s %s + %g * %s%s%s%s%s -> %s, %s k=%d parts=%d", (st.flags & MK_F_ONLY_MULTI) ? "[multi-token only]" : "", x.name.c_str(), st.alpha, yw ? "norm of " : "", y ? y->name.c_str() : "0", y2 ? " + " : "",
                              y2 ? y2->name.c_str() : "", st.conv_w ? " (+conv)" : "", no_xo ? "-" : xo.name.c_str(), o.name.c_str(), width, st.norm_groups));
  if (st.conv_w && B > 1) {
    g->stages.push_back(conv);
    g->stage_desc.push_back(conv_desc);
  }
  if (!fuse) return MK_OK;
  rc = lower_linear(g, i);
  if (rc) return rc;
  MkStage &l = g->stages.back();
  l.y_scale = st.y_scale;
  l.y2 = st.y2;
  l.ld_y2 = st.ld_y2;
  l.y2_scale = st.y2_scale;
  l.conv_w = st.conv_w;
  l.taps = st.taps;
  l.tail = st.tail;
  l.flags |= MK_F_NORM | MK_F_PRENORM | (st.flags & MK_F_RES_EARLY);
  l.y_in = st.in;
  l.ld_y = st.ld_in;
  l.y_norm_w = st.y_norm_w;
  l.in_bias = st.in_bias;
  l.slots = st.slots;
  l.ld_slot = st.ld_slot;
  l.slot_w = st.slot_w;
  l.ld_slot_w = st.ld_slot_w;
  l.res = st.res;
  l.ld_res = st.ld_res;
  l.norm_w = st.norm_w;
  l.norm_out = st.conv_w ? st.out3 : st.out;  // the rows its multi-token forms read
  l.ld_norm = st.conv_w ? st.ld_out3 : st.ld_out;
  l.out3 = st.conv_w ? st.out : nullptr;      // (the normed rows, which the single-token form writes)
  l.out2 = st.out2;
  l.ld_out2 = st.ld_out2;
  l.alpha = st.alpha;
  l.norm_groups = st.norm_groups;
  l.eps = st.eps;
  l.norm_eps = st.norm_eps;
  l.k_real = width;
  return MK_OK;
}

// gated activation beside another stage: params [output column, n, gate column, up column, limit bits, beta bits, bias bits]
int lower_glu(mk_graph *g, const Task &t, int out_op, size_t p, const Tensor &in, MkStage *st) {
  if (t.ops[out_op] < 0) return MK_OK;
  const Tensor &o = g->tensors[t.ops[out_op]];
  const int at = t.params[p], n = t.params[p + 1], a = t.params[p + 2], b = t.params[p + 3];
  if (at < 0 || at % 4 || n < 4 || n % 4 || a < 0 || b < 0 || a % 4 || b % 4 || a + n > in.dims[1] || b + n > in.dims[1] || !rows_ok(o, g->cfg.max_num_batched_tokens, at + n, in.dtype))
    return fail(MK_EINVAL, "%s: gated activation of %d columns at %d / %d does not fit its rows (multiples of 4)", t.name.c_str(), n, a, b);
  st->glu_out = (char *)o.ptr + (size_t)at * dtype_size(o.dtype);
  st->ld_glu = (int)o.strides[0];
  st->glu_n = n;
  st->glu_gate = a;
  st->glu_up = b;
  st->glu_limit = bits_f32(t.params[p + 4]);
  st->glu_beta = bits_f32(t.params[p + 5]);
  st->glu_bias = bits_f32(t.params[p + 6]);
  return MK_OK;
}

int lower_rotary_tables(mk_graph *g, const Task &t, int op, int rot, MkStage *st) {
  if (rot == 0) return MK_OK;
  if (t.ops[op] < 0 || t.ops[op + 1] < 0) return fail(MK_EINVAL, "%s: rotated dims without cos / sin tables", t.name.c_str());
  const Tensor &c = g->tensors[t.ops[op]], &s = g->tensors[t.ops[op + 1]];
  if (c.dtype != MK_DT_F32 || s.dtype != MK_DT_F32 || c.ndims != 2 || s.ndims != 2 || c.dims[1] != rot / 2 || s.dims[1] != rot / 2 || c.dims[0] < g->cfg.max_seq_length ||
      s.dims[0] < g->cfg.max_seq_length || c.strides[0] != s.strides[0])
    return fail(MK_EINVAL, "%s: cos / sin tables must be fp32 [>= max_seq_length, rotated dims / 2]", t.name.c_str());
  st->cos_tab = c.ptr;
  st->sin_tab = s.ptr;
  st->ld_cos = (int)c.strides[0];
  return MK_OK;
}

struct LatentDims {
  int kw, nrc, nkc, rp;
};
LatentDims latent_dims(int dtype, int rank, int rot) {
  LatentDims d;
  d.kw = dtype == MK_DT_F32 ? 16 : 32;
  d.nrc = (rank + d.kw - 1) / d.kw;
  d.nkc = d.nrc + (rot + d.kw - 1) / d.kw;
  d.rp = d.nrc * d.kw;
  return d;
}
int check_latent_cache(mk_graph *g, const Tensor &kc, int dtype, const LatentDims &d, const char *task) {
  if (kc.ndims != 3 || kc.dtype != dtype || kc.dims[0] < g->cfg.max_num_pages || kc.dims[1] != g->cfg.page_size || kc.dims[2] != d.nkc * d.kw)
    return fail(MK_EINVAL, "%s: the cache must be [>= %d pages, %d, %d], of the rows' type", task, g->cfg.max_num_pages, g->cfg.page_size, d.nkc * d.kw);
  return MK_OK;
}

// latent_prep [rows, q norm (fp32), latent norm (fp32, optional), cos (optional), sin (optional), cache (optional), activation
// (optional), q latents] params [q column, q rank, latent column, latent rank, rotated column, rotated dims, eps bits, then the
// gated activation's seven]
int lower_latent_prep(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 8 || t.params.size() != 14) return fail(MK_EINVAL, "latent_prep expects 8 operands / 14 params");
  const bool q = t.ops[1] >= 0;  // (without a query latent: operands 1 and 7 are absent)
  const Tensor &in = g->tensors[t.ops[0]];
  const int B = g->cfg.max_num_batched_tokens, qc = t.params[0], qr = t.params[1], kc = t.params[2], R = t.params[3], rc_ = t.params[4], rot = t.params[5];
  int rc = set_mix(g, in.dtype, "latent_prep");
  if (rc) return rc;
  auto up4 = [](int n) { return (n + 3) / 4 * 4; };
  if (q != (t.ops[7] >= 0) || (!q && (t.ops[5] < 0 || qr || !rows_ok(in, B, 4, in.dtype)))) return fail(MK_EINVAL, "latent_prep: nothing to do, or half a query latent");
  if (q && (qr < 1 || qc < 0 || qc % 4 || qr > MK_MX_MAX_NORM_ROW || !rows_ok(in, B, qc + up4(qr), in.dtype) || !rows_ok(g->tensors[t.ops[7]], B, up4(qr), in.dtype) || !vector_ok(g->tensors[t.ops[1]], up4(qr))))
    return fail(MK_EINVAL, "latent_prep: query latent of %d values at column %d (at most %d, columns multiples of 4, weights padded to 4)", qr, qc, MK_MX_MAX_NORM_ROW);
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_MX_LATENT_PREP;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.n = qr;
  st.cols[0] = qc;
  if (q) {
    st.q_norm_w = g->tensors[t.ops[1]].ptr;
    st.out = g->tensors[t.ops[7]].ptr;
    st.ld_out = (int)g->tensors[t.ops[7]].strides[0];
  }
  st.eps = bits_f32(t.params[6]);
  if (t.ops[5] >= 0) {
    const LatentDims d = latent_dims(in.dtype, R, rot);
    if (t.ops[2] < 0 || R < 1 || R > MK_MX_MAX_LATENT || kc < 0 || kc % 4 || rot < 0 || rot % 2 || rc_ < 0 || kc + up4(R) > in.dims[1] || rc_ + rot > in.dims[1] ||
        !vector_ok(g->tensors[t.ops[2]], up4(R)))
      return fail(MK_EINVAL, "latent_prep: latent of %d values (at most %d) at column %d, %d rotated at %d", R, MK_MX_MAX_LATENT, kc, rot, rc_);
    if ((rc = check_latent_cache(g, g->tensors[t.ops[5]], in.dtype, d, "latent_prep"))) return rc;
    if ((rc = lower_rotary_tables(g, t, 3, rot, &st))) return rc;
    st.k_cache = g->tensors[t.ops[5]].ptr;
    st.k_norm_w = g->tensors[t.ops[2]].ptr;
    st.rank = R;
    st.rot_dims = rot;
    st.cols[1] = kc;
    st.cols[2] = rc_;
  }
  if ((rc = lower_glu(g, t, 6, 7, in, &st))) return rc;
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MX_LATENT_PREP %s -> %s q=%d latent=%d rot=%d glu=%d", in.name.c_str(), q ? g->tensors[t.ops[7]].name.c_str() : "cache", qr, st.rank, st.rot_dims, st.glu_n));
  i++;
  return MK_OK;
}

// head_linear [rows, weights, ids (optional), table (optional), output] params [heads, n, k, input columns per head, output
// columns per head, table column]: one n x k matrix per head, weights in matrix-core operand order (see mk_mix.hip); with a
// table: out = gelu(.) * table[id][column + n].
int lower_head_linear(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 5 || t.params.size() != 6) return fail(MK_EINVAL, "head_linear expects 5 operands / 6 params");
  const Tensor &in = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &o = g->tensors[t.ops[4]];
  const int B = g->cfg.max_num_batched_tokens, H = t.params[0], n = t.params[1], k = t.params[2], is = t.params[3], os = t.params[4], tc = t.params[5];
  int rc = set_mix(g, in.dtype, "head_linear");
  if (rc) return rc;
  const int es = in.dtype == MK_DT_F32 ? 4 : 2, kw = 64 / es, epc = 16 / es;
  const bool out32 = o.dtype == MK_DT_F32 && in.dtype == MK_DT_BF16 && H == 1 && t.ops[3] < 0;  // 32-bit sums
  if (H < 1 || n < 1 || k < kw || k % kw || is < 0 || is % epc || os < 0 || in.strides[0] % epc || !rows_ok(in, B, (int64_t)(H - 1) * is + k, in.dtype) ||
      o.ndims != 2 || o.dims[0] < B || o.dims[1] < (int64_t)(H - 1) * os + n || (o.dtype != in.dtype && !out32) || w.dtype != in.dtype || (int64_t)w.elems() != (int64_t)H * ((n + 15) / 16 * 16) * k)
    return fail(MK_EINVAL, "head_linear: %d heads of %d x %d (whole operand rows of %d), input columns %d and output columns %d per head do not fit the operands", H, n, k, kw, is, os);
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_MX_HEAD_LINEAR;
  st.groups = H;
  st.n = n;
  st.k = k;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.ld_in_slot = is;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  st.ld_out_slot = os;
  st.w.nseg = 1;
  st.w.seg[0] = w.ptr;
  if (out32) {
    st.flags |= MK_F_OUT32;
    st.out2 = o.ptr;
    st.ld_out2 = (int)o.strides[0];
    g->hyb = true;
  }
  if (t.ops[3] >= 0) {
    const Tensor &tab = g->tensors[t.ops[3]];
    if (t.ops[2] < 0 || H != 1 || tab.ndims != 2 || tab.dtype != in.dtype || tc < 0 || tc + n > tab.dims[1] || g->tensors[t.ops[2]].dtype != MK_DT_I64 || (int64_t)g->tensors[t.ops[2]].elems() < B)
      return fail(MK_EINVAL, "head_linear: a table needs int64 ids, one per token row, one head and %d columns from %d on", n, tc);
    st.flags |= MK_F_GELU_TABLE;
    st.aux0 = g->tensors[t.ops[2]].ptr;
    st.aux1 = (char *)tab.ptr + (size_t)tc * es;
    st.ld_res = (int)tab.strides[0];
  }
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MX_HEAD_LINEAR %s x %s -> %s heads=%d n=%d k=%d%s", in.name.c_str(), w.name.c_str(), o.name.c_str(), H, n, k, t.ops[3] >= 0 ? " gelu * table" : ""));
  g->weight_bytes += (int64_t)w.elems() * es;
  i++;
  return MK_OK;
}

// latent_attention [query rows, query latents, cache, cos (optional), sin (optional), output] params [heads, latent rank, rotated
// dims, query columns per head, rotated column of a head, scale bits]
int lower_latent_attention(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 6 || t.params.size() != 6) return fail(MK_EINVAL, "latent_attention expects 6 operands / 6 params");
  const Tensor &q = g->tensors[t.ops[0]], &ql = g->tensors[t.ops[1]], &kc = g->tensors[t.ops[2]], &o = g->tensors[t.ops[5]];
  const int B = g->cfg.max_num_batched_tokens, ps = g->cfg.page_size, H = t.params[0], R = t.params[1], rot = t.params[2], hs = t.params[3], ro = t.params[4];
  int rc = set_mix(g, q.dtype, "latent_attention");
  if (rc) return rc;
  const bool f32 = q.dtype == MK_DT_F32;
  if (H < 1 || R < 1 || R > MK_MX_MAX_LATENT || rot < 0 || rot % 2) return fail(MK_EINVAL, "latent_attention: %d heads, latent of %d values (at most %d), %d rotated", H, R, MK_MX_MAX_LATENT, rot);
  const LatentDims d = latent_dims(q.dtype, R, rot);
  if (hs < 0 || ro < 0 || !rows_ok(q, B, (int64_t)(H - 1) * hs + ro + rot, q.dtype) || !rows_ok(ql, B, (int64_t)H * d.rp, q.dtype) || (ql.strides[0] * (f32 ? 4 : 2)) % 16 || !rows_ok(o, B, (int64_t)H * d.rp, q.dtype))
    return fail(MK_EINVAL, "latent_attention: query latents and output are [tokens, >= heads * %d], the query rows hold %d columns per head", d.rp, hs);
  if ((rc = check_latent_cache(g, kc, q.dtype, d, "latent_attention"))) return rc;
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_MX_LATENT_ATTN;
  st.in = q.ptr;
  st.ld_in = (int)q.strides[0];
  st.ld_in_slot = hs;
  st.cols[0] = ro;
  st.q_ws = ql.ptr;
  st.ld_qws = (int)ql.strides[0];
  st.k_cache = kc.ptr;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  st.num_q_heads = H;
  st.rank = R;
  st.rot_dims = rot;
  st.sm_scale = bits_f32(t.params[5]);
  if ((rc = lower_rotary_tables(g, t, 3, rot, &st))) return rc;
  // instantiation (mk_mix.hip: stage_mx_latent_attn): operand rows of a cached latent, 16-position sub-tiles of a tile, 16-row
  // query tiles of a unit
  st.nk = f32 ? (R <= 128 && d.nkc <= 12 ? 12 : 40) : (R <= 128 && d.nkc <= 6 ? 6 : d.nkc <= 18 ? 18 : 20);
  st.k_tiles = f32 ? 2 : 4;
  st.v_tiles = f32 ? 1 : 2;
  if (d.nkc > st.nk) return fail(MK_EUNSUPPORTED, "latent_attention: latent of %d and rotated part of %d values (%d operand rows, at most %d)", R, rot, d.nkc, st.nk);
  if (ps % (16 * st.k_tiles)) return fail(MK_EINVAL, "latent_attention: page_size %d must be a multiple of %d", ps, 16 * st.k_tiles);
  const int pages = (g->cfg.max_seq_length + ps - 1) / ps;
  if (mk_latent_lds(f32 ? 4 : 2, st.v_tiles, st.nk, st.k_tiles, pages).bytes > MK_LDS_BYTES) return fail(MK_EUNSUPPORTED, "latent_attention: %d pages per request need too much LDS", pages);
  g->flex_part = std::max(g->flex_part, (size_t)g->G * 16 * st.v_tiles * (d.rp + 32));
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MX_LATENT_ATTN %s, %s -> %s heads=%d latent=%d rot=%d scale=%g", q.name.c_str(), ql.name.c_str(), o.name.c_str(), H, R, rot, st.sm_scale));
  st.op = MK_OP_MX_LATENT_MERGE;
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MX_LATENT_MERGE[split requests] -> %s", o.name.c_str()));
  i++;
  return MK_OK;
}

// general_delta [rows, decay weights, decay offset (fp32), removal offset (fp32), norm (fp32), state (fp32), state slots (int32),
// workspace (fp32), activation (optional), output] params [heads, dim, low rank (whole operand rows), columns of r k v g a and the
// low-rank projection, eps bits, then the gated activation's seven].  A head's columns, offsets, norm and output are dim rounded
// up to 16 wide; the workspace rows hold twice that for all heads.
int lower_general_delta(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 10 || t.params.size() != 17) return fail(MK_EINVAL, "general_delta expects 10 operands / 17 params");
  const Tensor &in = g->tensors[t.ops[0]], &w2 = g->tensors[t.ops[1]], &state = g->tensors[t.ops[5]], &ids = g->tensors[t.ops[6]], &ws = g->tensors[t.ops[7]], &o = g->tensors[t.ops[9]];
  const int B = g->cfg.max_num_batched_tokens, slots = g->cfg.max_num_batched_requests, H = t.params[0], D = t.params[1], rank = t.params[2];
  int rc = set_mix(g, in.dtype, "general_delta");
  if (rc) return rc;
  const int es = in.dtype == MK_DT_F32 ? 4 : 2, kw = 64 / es;
  if (H < 1 || D < 1 || D > MK_MX_MAX_DELTA_DIM || rank < kw || rank % kw || rank > MK_MX_MAX_RANK)
    return fail(MK_EUNSUPPORTED, "general_delta: %d heads of %d (at most %d), low rank %d (whole operand rows of %d, at most %d)", H, D, MK_MX_MAX_DELTA_DIM, rank, kw, MK_MX_MAX_RANK);
  const int dp = (D + 15) / 16 * 16, cols = H * dp;
  if (!rows_ok(in, B, 1, in.dtype) || (in.strides[0] * es) % 16 || !rows_ok(o, B, cols, in.dtype) || !rows_ok(ws, B, 2 * (int64_t)cols, MK_DT_F32)) return fail(MK_EINVAL, "general_delta: bad row tensors");
  for (int a = 0; a < 6; a++) {
    const int col = t.params[3 + a], n = a == 5 ? rank : cols;
    if (col < 0 || col % (16 / es) || col + n > in.dims[1]) return fail(MK_EINVAL, "general_delta: columns %d .. %d lie outside the rows or begin inside a 16-byte word", col, col + n);
  }
  if (w2.dtype != in.dtype || (int64_t)w2.elems() != (int64_t)cols * rank || !vector_ok(g->tensors[t.ops[2]], cols) || !vector_ok(g->tensors[t.ops[3]], cols) || !vector_ok(g->tensors[t.ops[4]], cols))
    return fail(MK_EINVAL, "general_delta: decay weights are %d x %d in operand order, the three vectors fp32 of %d", cols, rank, cols);
  if (state.dtype != MK_DT_F32 || state.ndims != 4 || state.dims[0] < slots || state.dims[1] != H || state.dims[2] != dp || state.dims[3] != dp)
    return fail(MK_EINVAL, "general_delta: the state is fp32 [>= %d slots, %d, %d, %d]", slots, H, dp, dp);
  if (ids.dtype != MK_DT_I32 || (int)ids.elems() < slots) return fail(MK_EINVAL, "general_delta: one int32 state slot per batch slot");
  if (g->state_ids && g->state_ids != (int *)ids.ptr) return fail(MK_EINVAL, "general_delta: every recurrence of a graph uses the same state-slot tensor");
  g->state_ids = (int *)ids.ptr;
  MkStage sd;  // decays
  memset(&sd, 0, sizeof(sd));
  sd.op = MK_OP_MX_DECAY;
  sd.groups = 1;
  sd.n = cols;
  sd.k = rank;
  sd.in = (const char *)in.ptr + (size_t)t.params[8] * es;
  sd.ld_in = (int)in.strides[0];
  sd.w.nseg = 1;
  sd.w.seg[0] = w2.ptr;
  sd.q_norm_w = g->tensors[t.ops[2]].ptr;
  sd.out2 = ws.ptr;
  sd.ld_out2 = (int)ws.strides[0];
  if ((rc = lower_glu(g, t, 8, 10, in, &sd))) return rc;
  sd.glu_gate -= t.params[8];  // (columns from the low-rank projection on)
  sd.glu_up -= t.params[8];
  g->stages.push_back(sd);
  g->stage_desc.push_back(fmt("MX_DECAY %s x %s n=%d k=%d glu=%d", in.name.c_str(), w2.name.c_str(), cols, rank, sd.glu_n));
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_MX_DELTA;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.in2 = ws.ptr;
  st.ld_in2 = (int)ws.strides[0];
  st.out2 = (float *)ws.ptr + cols;
  st.ld_out2 = (int)ws.strides[0];
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  st.num_q_heads = H;
  st.head_dim = D;
  for (int a = 0; a < 5; a++) st.cols[a] = t.params[3 + a];
  st.eps = bits_f32(t.params[9]);
  st.k_norm_w = g->tensors[t.ops[3]].ptr;
  st.norm_w = g->tensors[t.ops[4]].ptr;
  st.k_cache = state.ptr;
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MX_DELTA %s -> %s heads=%d d=%d", in.name.c_str(), o.name.c_str(), H, D));
  st.op = MK_OP_MX_DELTA_OUT;
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MX_DELTA_OUT[sliced] -> %s", o.name.c_str()));
  g->weight_bytes += (int64_t)w2.elems() * es;
  i++;
  return MK_OK;
}

// ---- hybrid tasks (mk_hybrid.hip) --------------------------------------------------------------------------------------
int set_hyb(mk_graph *g, int dtype, const char *task) {
  g->hyb = true;
  return set_mix(g, dtype, task);
}
int set_state_slots(mk_graph *g, const Tensor &ids, const char *task) {
  if (ids.dtype != MK_DT_I32 || (int)ids.elems() < g->cfg.max_num_batched_requests) return fail(MK_EINVAL, "%s: one int32 state slot per batch slot", task);
  if (g->state_ids && g->state_ids != (int *)ids.ptr) return fail(MK_EINVAL, "%s: every recurrence of a graph uses the same state-slot tensor", task);
  g->state_ids = (int *)ids.ptr;
  return MK_OK;
}
bool tail_ok(const mk_graph *g, const Tensor &t, int taps, int n, int dtype) {
  return t.ndims == 3 && t.dtype == dtype && t.dims[0] >= g->cfg.max_num_batched_requests && t.dims[1] >= (taps > 1 ? taps - 1 : 1) && t.dims[2] == n && t.strides[1] == n &&
         (taps == 1 || t.dims[1] == taps - 1);
}

// short_conv [rows, weights (fp32 [taps, channels]), bias (fp32), tail, state slots (int32), output] params [column]
int lower_short_conv(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 6 || t.params.size() != 1) return fail(MK_EINVAL, "short_conv expects 6 operands / 1 param");
  const Tensor &in = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &b = g->tensors[t.ops[2]], &tail = g->tensors[t.ops[3]], &o = g->tensors[t.ops[5]];
  const int B = g->cfg.max_num_batched_tokens, col = t.params[0], taps = w.ndims == 2 ? (int)w.dims[0] : 0, n = w.ndims == 2 ? (int)w.dims[1] : 0;
  int rc = set_hyb(g, in.dtype, "short_conv");
  if (rc) return rc;
  if (taps < 1 || n < 4 || n % 4 || col < 0 || col % 4 || w.dtype != MK_DT_F32 || w.strides[0] != n || !vector_ok(b, n) || !rows_ok(in, B, (int64_t)col + n, in.dtype) || !rows_ok(o, B, n, in.dtype) ||
      !tail_ok(g, tail, taps, n, in.dtype))
    return fail(MK_EINVAL, "short_conv: %d taps over %d channels (a multiple of 4) at column %d do not fit the operands", taps, n, col);
  if ((rc = set_state_slots(g, g->tensors[t.ops[4]], "short_conv"))) return rc;
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_HY_CONV;
  st.n = n;
  st.taps = taps;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.cols[0] = col;
  st.norm_w = w.ptr;
  st.in_bias = (const float *)b.ptr;
  st.tail = tail.ptr;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("HY_CONV %s -> %s n=%d taps=%d", in.name.c_str(), o.name.c_str(), n, taps));
  i++;
  return MK_OK;
}

// ring_conv [rows, weights [taps, channels], bias (fp32, optional), ring [slots, taps, channels], state slots (int32), step bias (fp32 [heads],
// optional), log2(e) x rates (fp32 [heads]), output, steps and decays (fp32, optional)] params [column, silu 0/1, identity 0/1, heads, step
// column, column of the decays]: see stage_du_conv.
int lower_ring_conv(mk_graph *g, size_t &i, MkStage *to, std::string *desc) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 9 || t.params.size() != 6) return fail(MK_EINVAL, "ring_conv expects 9 operands / 6 params");
  const Tensor &in = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &ring = g->tensors[t.ops[3]], &o = g->tensors[t.ops[7]];
  const Tensor *b = t.ops[2] >= 0 ? &g->tensors[t.ops[2]] : nullptr, *sb = t.ops[5] >= 0 ? &g->tensors[t.ops[5]] : nullptr;
  const int B = g->cfg.max_num_batched_tokens, col = t.params[0], taps = w.ndims == 2 ? (int)w.dims[0] : 0, n = w.ndims == 2 ? (int)w.dims[1] : 0, H = t.params[3], scol = t.params[4], dcol = t.params[5];
  int rc = set_hyb(g, in.dtype, "ring_conv");
  if (rc) return rc;
  g->dual = true;
  if (taps > MK_DU_MAX_TAPS) return fail(MK_EUNSUPPORTED, "ring_conv: %d taps (at most %d)", taps, MK_DU_MAX_TAPS);
  if (taps < 1 || n < 4 || n % 4 || col < 0 || col % 4 || w.dtype != in.dtype || w.strides[0] != n || (b && !vector_ok(*b, n)) || !rows_ok(in, B, (int64_t)col + n, in.dtype) || !rows_ok(o, B, n, in.dtype) ||
      o.ptr == in.ptr || ring.ndims != 3 || ring.dtype != in.dtype || ring.dims[0] < g->cfg.max_num_batched_requests || ring.dims[1] != taps || ring.dims[2] != n || ring.strides[0] != (int64_t)taps * n || ring.strides[1] != n)
    return fail(MK_EINVAL, "ring_conv: %d taps over %d channels (a multiple of 4) at column %d do not fit the operands", taps, n, col);
  if (sb && (t.ops[6] < 0 || t.ops[8] < 0 || H < 1 || scol < 0 || scol + H > in.dims[1] || dcol < H || !vector_ok(*sb, H) || !vector_ok(g->tensors[t.ops[6]], H) || !rows_ok(g->tensors[t.ops[8]], B, (int64_t)dcol + H, MK_DT_F32)))
    return fail(MK_EINVAL, "ring_conv: %d steps at column %d, decays from column %d on, do not fit the operands", H, scol, dcol);
  if ((rc = set_state_slots(g, g->tensors[t.ops[4]], "ring_conv"))) return rc;
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_DU_CONV;
  if (t.params[1]) st.flags |= MK_F_SILU;
  if (t.params[2]) st.flags |= MK_F_IDENTITY;
  st.n = n;
  st.taps = taps;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.cols[0] = col;
  st.conv_w = w.ptr;
  st.in_bias = b ? (const float *)b->ptr : nullptr;
  st.tail = ring.ptr;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  if (sb) {
    st.num_q_heads = H;
    st.step_bias = (const float *)sb->ptr;
    st.a_tab = (const float *)g->tensors[t.ops[6]].ptr;
    st.cols[1] = scol;
    st.cols[2] = dcol;
    st.out2 = g->tensors[t.ops[8]].ptr;
    st.ld_out2 = (int)g->tensors[t.ops[8]].strides[0];
  }
  const std::string d = fmt("DU_CONV%s %s -> %s n=%d taps=%d steps=%d", to ? "[portions]" : "", in.name.c_str(), o.name.c_str(), n, taps, sb ? H : 0);
  if (to) {
    *to = st;
    *desc = d;
  } else {
    g->stages.push_back(st);
    g->stage_desc.push_back(d);
  }
  i++;
  return MK_OK;
}

// dual_scan [rows, convolved rows, steps and decays (fp32), D (fp32 [heads]), state (fp32), state slots (int32), output (fp32)] params [heads,
// values per head, states, groups, z column of the rows, x, B and C column of the convolved rows, column of the decays]
int lower_dual_scan(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 7 || t.params.size() != 9) return fail(MK_EINVAL, "dual_scan expects 7 operands / 9 params");
  const Tensor &in = g->tensors[t.ops[0]], &xc = g->tensors[t.ops[1]], &dt = g->tensors[t.ops[2]], &D = g->tensors[t.ops[3]], &state = g->tensors[t.ops[4]], &o = g->tensors[t.ops[6]];
  const int B = g->cfg.max_num_batched_tokens, H = t.params[0], V = t.params[1], N = t.params[2], G = t.params[3], zc = t.params[4], x0 = t.params[5], b0 = t.params[6], c0 = t.params[7], dc = t.params[8], np = (N + 3) / 4 * 4;
  int rc = set_hyb(g, in.dtype, "dual_scan");
  if (rc) return rc;
  g->dual = true;
  if (N < 1 || N > MK_HY_MAX_STATES || H < 1 || V < 1 || G < 1 || H % G) return fail(MK_EUNSUPPORTED, "dual_scan: %d heads of %d values in %d groups, %d states (at most %d)", H, V, G, N, MK_HY_MAX_STATES);
  if (zc < 0 || x0 < 0 || b0 < 0 || b0 % 4 || c0 < 0 || c0 % 4 || dc < H || !vector_ok(D, H) || !rows_ok(in, B, (int64_t)zc + (int64_t)H * V, in.dtype) ||
      !rows_ok(xc, B, std::max((int64_t)x0 + (int64_t)H * V, (int64_t)std::max(b0, c0) + (int64_t)G * np), in.dtype) || !rows_ok(dt, B, (int64_t)dc + H, MK_DT_F32) || !rows_ok(o, B, (int64_t)H * V, MK_DT_F32))
    return fail(MK_EINVAL, "dual_scan: %d heads of %d values, %d groups of %d states do not fit the operands", H, V, G, N);
  if (state.dtype != MK_DT_F32 || state.ndims != 4 || state.dims[0] < g->cfg.max_num_batched_requests || state.dims[1] != H || state.dims[2] != V || state.dims[3] != np || state.strides[2] != np ||
      state.strides[1] != (int64_t)V * np || state.strides[0] != (int64_t)H * V * np)
    return fail(MK_EINVAL, "dual_scan: the state is fp32 [>= %d slots, %d, %d, %d]", g->cfg.max_num_batched_requests, H, V, np);
  if ((rc = set_state_slots(g, g->tensors[t.ops[5]], "dual_scan"))) return rc;
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_DU_SCAN;
  st.num_q_heads = H;
  st.v_dim = V;
  st.states = N;
  st.groups = G;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.cols[0] = x0;
  st.cols[1] = b0;
  st.cols[2] = c0;
  st.cols[3] = zc;
  st.cols[4] = dc;
  st.q_ws = xc.ptr;
  st.ld_qws = (int)xc.strides[0];
  st.in2 = dt.ptr;
  st.ld_in2 = (int)dt.strides[0];
  st.d_tab = (const float *)D.ptr;
  st.k_cache = state.ptr;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("DU_SCAN %s -> %s heads=%d n=%d states=%d groups=%d", xc.name.c_str(), o.name.c_str(), H, V, N, G));
  i++;
  return MK_OK;
}

// scan_step [rows, weights (operand order), offset (fp32), output (fp32)] params [n, k, column]: softplus(W x + offset)
int lower_scan_step(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 4 || t.params.size() != 3) return fail(MK_EINVAL, "scan_step expects 4 operands / 3 params");
  const Tensor &in = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &b = g->tensors[t.ops[2]], &o = g->tensors[t.ops[3]];
  const int B = g->cfg.max_num_batched_tokens, n = t.params[0], k = t.params[1], col = t.params[2];
  int rc = set_hyb(g, in.dtype, "scan_step");
  if (rc) return rc;
  const int es = in.dtype == MK_DT_F32 ? 4 : 2, kw = 64 / es, epc = 16 / es;
  if (n < 16 || n % 16 || k < kw || k % kw || col < 0 || col % epc || in.strides[0] % epc || !rows_ok(in, B, (int64_t)col + k, in.dtype) || !rows_ok(o, B, n, MK_DT_F32) || !vector_ok(b, n) ||
      w.dtype != in.dtype || (int64_t)w.elems() != (int64_t)n * k)
    return fail(MK_EINVAL, "scan_step: %d x %d weights (multiples of 16 and %d) at column %d do not fit the operands", n, k, kw, col);
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_HY_STEP;
  st.groups = 1;
  st.n = n;
  st.k = k;
  st.in = (const char *)in.ptr + (size_t)col * es;
  st.ld_in = (int)in.strides[0];
  st.w.nseg = 1;
  st.w.seg[0] = w.ptr;
  st.in_bias = (const float *)b.ptr;
  st.out2 = o.ptr;
  st.ld_out2 = (int)o.strides[0];
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("HY_STEP %s x %s -> %s n=%d k=%d", in.name.c_str(), w.name.c_str(), o.name.c_str(), n, k));
  g->weight_bytes += (int64_t)w.elems() * es;
  i++;
  return MK_OK;
}

// selective_scan [rows, convolved rows, step sizes (fp32), B / C rows, A (fp32 [channels, states up to 4]), D (fp32), state (fp32), tail,
// state slots (int32), output] params [states, taps, x column, z column of the rows, B column, C column of the B / C rows]
int lower_selective_scan(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 10 || t.params.size() != 6) return fail(MK_EINVAL, "selective_scan expects 10 operands / 6 params");
  const Tensor &in = g->tensors[t.ops[0]], &xc = g->tensors[t.ops[1]], &dt = g->tensors[t.ops[2]], &bc = g->tensors[t.ops[3]], &A = g->tensors[t.ops[4]], &D = g->tensors[t.ops[5]],
               &state = g->tensors[t.ops[6]], &tail = g->tensors[t.ops[7]], &o = g->tensors[t.ops[9]];
  const int B = g->cfg.max_num_batched_tokens, N = t.params[0], taps = t.params[1], xcol = t.params[2], zcol = t.params[3], bcol = t.params[4], ccol = t.params[5], np = (N + 3) / 4 * 4;
  int rc = set_hyb(g, in.dtype, "selective_scan");
  if (rc) return rc;
  const int n = A.ndims == 2 ? (int)A.dims[0] : 0;
  if (N < 1 || N > MK_HY_MAX_STATES || taps < 1 || n < 4) return fail(MK_EUNSUPPORTED, "selective_scan: %d channels, %d states (at most %d), %d taps", n, N, MK_HY_MAX_STATES, taps);
  if (A.dtype != MK_DT_F32 || A.dims[1] != np || A.strides[0] != np || !vector_ok(D, n) || xcol < 0 || zcol < 0 || bcol < 0 || ccol < 0 || bcol % 4 || ccol % 4 ||
      !rows_ok(in, B, (int64_t)std::max(xcol, zcol) + n, in.dtype) || !rows_ok(xc, B, n, in.dtype) || !rows_ok(dt, B, n, MK_DT_F32) || !rows_ok(bc, B, (int64_t)std::max(bcol, ccol) + np, in.dtype) ||
      !rows_ok(o, B, n, in.dtype) || !tail_ok(g, tail, taps, n, in.dtype))
    return fail(MK_EINVAL, "selective_scan: %d channels of %d states and %d taps do not fit the operands", n, N, taps);
  if (state.dtype != MK_DT_F32 || state.ndims != 3 || state.dims[0] < g->cfg.max_num_batched_requests || state.dims[1] != n || state.dims[2] != np || state.strides[1] != np)
    return fail(MK_EINVAL, "selective_scan: the state is fp32 [>= %d slots, %d, %d]", g->cfg.max_num_batched_requests, n, np);
  if ((rc = set_state_slots(g, g->tensors[t.ops[8]], "selective_scan"))) return rc;
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_HY_SCAN;
  st.n = n;
  st.states = N;
  st.taps = taps;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.cols[0] = xcol;
  st.cols[1] = bcol;
  st.cols[2] = ccol;
  st.cols[3] = zcol;
  st.q_ws = xc.ptr;
  st.ld_qws = (int)xc.strides[0];
  st.in2 = dt.ptr;
  st.ld_in2 = (int)dt.strides[0];
  st.in3 = bc.ptr;
  st.ld_in3 = (int)bc.strides[0];
  st.a_tab = (const float *)A.ptr;
  st.d_tab = (const float *)D.ptr;
  st.k_cache = state.ptr;
  st.tail = tail.ptr;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("HY_SCAN %s -> %s n=%d states=%d taps=%d", in.name.c_str(), o.name.c_str(), n, N, taps));
  i++;
  return MK_OK;
}

// expert_route [logits (fp32), ids (int32 [tokens, top]), shares (fp32)] params [experts, top, shared 0/1]: the stage runs for
// iterations of several tokens; the expert_linear behind it routes a single one itself.  With one more operand behind the logits (correction,
// fp32 [experts]) and three more params [groups, groups kept, scale bits]: sigmoid scores, choices among the best groups (MK_F_GROUPS); the
// shared expert's share is 1 and has no logit.
// expert_linear [rows, weights, shared weights (optional), ids, output] params [experts, top, n, k, shared n, shared k, gated 0/1, input
// columns per place (0: one row for all), output columns per place]; four more params [limit, beta, bias, shared expert's limit; bits]: the
// clamped activation (MK_F_CLAMP_GLU).
bool route_ok(int experts, int top) { return experts >= 1 && experts <= MK_MOE_MAX_EXPERTS && top >= 1 && top <= experts && top <= MK_MOE_MAX_TOPK; }
int lower_expert_route(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  const bool ext = t.ops.size() == 4 && t.params.size() == 6;
  if (!ext && (t.ops.size() != 3 || t.params.size() != 3)) return fail(MK_EINVAL, "expert_route expects 3 operands / 3 params, or 4 / 6");
  const Tensor &z = g->tensors[t.ops[0]], &ids = g->tensors[t.ops[1 + ext]], &w = g->tensors[t.ops[2 + ext]];
  const int ids_id = t.ops[1 + ext];
  const int B = g->cfg.max_num_batched_tokens, E = t.params[0], top = t.params[1], sh = t.params[2] ? 1 : 0;
  if (ext) {
    const int groups = t.params[3], keep = t.params[4];
    if (groups < 1 || E % groups || keep < 1 || keep > groups || top > keep * (E / groups) || !vector_ok(g->tensors[t.ops[1]], E))
      return fail(MK_EINVAL, "expert_route: %d of %d experts in %d groups of which %d stay open, a correction per expert", top, E, groups, keep);
    g->dual = true;
  }
  g->mix = g->hyb = true;
  if (!route_ok(E, top)) return fail(MK_EUNSUPPORTED, "expert_route: %d of %d experts (at most %d of %d)", top, E, MK_MOE_MAX_TOPK, MK_MOE_MAX_EXPERTS);
  if (!rows_ok(z, B, E + (ext ? 0 : sh), MK_DT_F32) || ids.ndims != 2 || ids.dtype != MK_DT_I32 || ids.dims[0] < B || ids.dims[1] != top || ids.strides[0] != top || !rows_ok(w, B, top + sh, MK_DT_F32))
    return fail(MK_EINVAL, "expert_route: logits fp32 [tokens, %d], ids int32 [tokens, %d], shares fp32 [tokens, >= %d]", E + sh, top, top + sh);
  if (i + 1 >= g->ltasks.size() || g->ltasks[i + 1].name != "expert_linear" || g->ltasks[i + 1].ops.size() != 5 || g->ltasks[i + 1].ops[3] != ids_id ||
      (g->ltasks[i + 1].ops[2] >= 0) != (sh != 0))
    return fail(MK_EUNSUPPORTED, "expert_route is followed by the expert_linear that reads its ids");
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_HY_ROUTE;
  st.flags = MK_F_ONLY_MULTI;
  st.num_experts = E;
  st.topk = top;
  st.moe_logits = z.ptr;
  st.ld_logits = (int)z.strides[0];
  st.ids = (int *)ids.ptr;
  st.slot_w = (const float *)w.ptr;
  st.ld_slot_w = (int)w.strides[0];
  st.w_shared = sh ? z.ptr : nullptr;  // (only its presence counts here)
  if (ext) {
    st.flags |= MK_F_GROUPS;
    st.choice_bias = (const float *)g->tensors[t.ops[1]].ptr;
    st.groups = t.params[3];
    st.groups_keep = t.params[4];
    st.choice_scale = bits_f32(t.params[5]);
  }
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("HY_ROUTE[multi-token only] %s -> %s experts=%d top=%d shared=%d", z.name.c_str(), w.name.c_str(), E, top, sh));
  i++;
  return MK_OK;
}
int lower_expert_linear(mk_graph *g, size_t &i) {
  const Task &t = g->ltasks[i];
  const bool clamp = t.params.size() == 13;
  if (t.ops.size() != 5 || (!clamp && t.params.size() != 9)) return fail(MK_EINVAL, "expert_linear expects 5 operands / 9 or 13 params");
  const Tensor &in = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &ids = g->tensors[t.ops[3]], &o = g->tensors[t.ops[4]];
  const Tensor *ws = t.ops[2] >= 0 ? &g->tensors[t.ops[2]] : nullptr;
  const int B = g->cfg.max_num_batched_tokens, E = t.params[0], top = t.params[1], n = t.params[2], k = t.params[3], ns = ws ? t.params[4] : 0, ks = ws ? t.params[5] : 0, glu = t.params[6] ? 2 : 1,
            is = t.params[7], os = t.params[8];
  int rc = set_hyb(g, in.dtype, "expert_linear");
  if (rc) return rc;
  const int es = in.dtype == MK_DT_F32 ? 4 : 2, kw = 64 / es, epc = 16 / es;
  auto up32 = [](int64_t x) { return (x + 31) / 32 * 32; };
  const int last = top + (ws ? 1 : 0) - 1;
  if (!route_ok(E, top)) return fail(MK_EUNSUPPORTED, "expert_linear: %d of %d experts (at most %d of %d)", top, E, MK_MOE_MAX_TOPK, MK_MOE_MAX_EXPERTS);
  if (n < 1 || k < kw || k % kw || is < 0 || is % epc || os < 4 || os % 4 || in.strides[0] % epc || (glu == 2 && (n % 32 || ns % 32)) || (ws && (ns < 1 || ks < kw || ks % kw)) ||
      !rows_ok(in, B, (int64_t)last * is + std::max(k, ks), in.dtype) || !rows_ok(o, B, (int64_t)last * os + std::max(n, ns) / glu, in.dtype) || os < std::max(n, ns) / glu ||
      w.dtype != in.dtype || (int64_t)w.elems() != E * up32(n) * k || (ws && (ws->dtype != in.dtype || (int64_t)ws->elems() != up32(ns) * ks)))
    return fail(MK_EINVAL, "expert_linear: %d experts of %d x %d (reductions in whole operand rows of %d, outputs padded to 32 rows), a shared one of %d x %d, do not fit the operands", E, n, k, kw, ns, ks);
  if (ids.ndims != 2 || ids.dtype != MK_DT_I32 || ids.dims[0] < B || ids.dims[1] != top || ids.strides[0] != top) return fail(MK_EINVAL, "expert_linear: ids are int32 [tokens, %d]", top);
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_HY_EXPERTS;
  if (glu == 2) st.flags |= MK_F_SILU;
  if (clamp) {
    if (glu != 2) return fail(MK_EINVAL, "expert_linear: the clamped activation belongs to a gated linear");
    g->dual = true;
    st.flags |= MK_F_CLAMP_GLU;
    st.glu_limit = bits_f32(t.params[9]);
    st.glu_beta = bits_f32(t.params[10]);
    st.glu_bias = bits_f32(t.params[11]);
    st.glu_limit_shared = bits_f32(t.params[12]);
  }
  st.num_experts = E;
  st.topk = top;
  st.n = n;
  st.k = k;
  st.n_shared = ns;
  st.k_shared = ks;
  st.in = in.ptr;
  st.ld_in = (int)in.strides[0];
  st.ld_in_slot = is;
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  st.ld_out_slot = os;
  st.w.nseg = 1;
  st.w.seg[0] = w.ptr;
  st.w_shared = ws ? ws->ptr : nullptr;
  st.ids = (int *)ids.ptr;
  if (!g->stages.empty() && g->stages.back().op == MK_OP_HY_ROUTE && g->stages.back().ids == st.ids) {
    const MkStage &r = g->stages.back();
    if (r.num_experts != E) return fail(MK_EINVAL, "expert_linear: %d experts, the routing has %d", E, r.num_experts);
    st.flags |= MK_F_MOE_INLINE_TOPK;
    st.moe_logits = r.moe_logits;
    st.ld_logits = r.ld_logits;
    st.slot_w = r.slot_w;
    st.ld_slot_w = r.ld_slot_w;
    st.flags |= r.flags & MK_F_GROUPS;
    st.choice_bias = r.choice_bias;
    st.groups = r.groups;
    st.groups_keep = r.groups_keep;
    st.choice_scale = r.choice_scale;
  }
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("HY_EXPERTS%s%s %s -> %s experts=%d top=%d n=%d k=%d shared=%dx%d", (st.flags & MK_F_MOE_INLINE_TOPK) ? "+route" : "", clamp ? "+clamped" : glu == 2 ? "+silu" : "", in.name.c_str(), o.name.c_str(), E,
                              top, n, k, ns, ks));
  g->weight_bytes += ((int64_t)top * n * k + (int64_t)ns * ks) * es;
  i++;
  return MK_OK;
}

bool is_moe_linear(const std::string &n) {
  return n == "moe_w13_linear_mi300" || n == "moe_w2_linear_mi300" || n == "gang_moe_w13_linear_mi300" || n == "gang_moe_w2_linear_mi300";
}

// dims 0 and 1 of a [tokens, topk, width] tensor must form one contiguous run of rows
bool rows_contiguous_3d(const Tensor &t) { return t.ndims == 3 && t.strides[2] == 1 && t.strides[0] == t.dims[1] * t.strides[1]; }

// Router: moe_topk_softmax_mi300 [logits, topk_weight, routing_indices, mask].  When the per-expert linear that consumes
// the routing follows directly, single-token iterations route inside that linear and this stage runs for multi-token
// iterations only.
int lower_moe_topk(mk_graph *g, size_t &i, bool *inline_next) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 4) return fail(MK_EINVAL, "%s expects 4 operands", t.name.c_str());
  const Tensor &lg = g->tensors[t.ops[0]], &tw = g->tensors[t.ops[1]], &ri = g->tensors[t.ops[2]], &mk = g->tensors[t.ops[3]];
  const int B = g->cfg.max_num_batched_tokens;
  if (lg.ndims != 2 || lg.dtype != MK_DT_BF16 || lg.dims[0] < B) return fail(MK_EINVAL, "%s: logits must be [tokens, experts] bf16", t.name.c_str());
  const int E = (int)lg.dims[1];
  if (E < 1 || E > MK_MOE_MAX_EXPERTS) return fail(MK_EUNSUPPORTED, "%s: %d experts (max %d)", t.name.c_str(), E, MK_MOE_MAX_EXPERTS);
  if (tw.ndims != 2 || tw.dtype != MK_DT_F32 || tw.dims[0] < B || tw.strides[1] != 1) return fail(MK_EINVAL, "%s: routing weights must be [tokens, topk] fp32", t.name.c_str());
  const int topk = (int)tw.dims[1];
  if (topk < 1 || topk > MK_MOE_MAX_TOPK || topk > E) return fail(MK_EUNSUPPORTED, "%s: top-%d of %d experts (max %d)", t.name.c_str(), topk, E, MK_MOE_MAX_TOPK);
  if (ri.ndims != 2 || ri.dtype != MK_DT_I32 || ri.dims[0] != E || ri.dims[1] < B || ri.strides[1] != 1)
    return fail(MK_EINVAL, "%s: routing indices must be [experts, tokens] int32", t.name.c_str());
  if (mk.dtype != MK_DT_I32 || mk.elems() < (size_t)E + 1) return fail(MK_EINVAL, "%s: mask must hold experts+1 int32", t.name.c_str());
  if (i + 1 >= g->ltasks.size() || !is_moe_linear(g->ltasks[i + 1].name) || g->ltasks[i + 1].ops.size() != 5 || g->ltasks[i + 1].ops[2] != t.ops[2] ||
      g->ltasks[i + 1].ops[3] != t.ops[3])
    return fail(MK_EUNSUPPORTED, "%s must be followed by the per-expert linear that consumes its routing table (it publishes the active-expert mask)", t.name.c_str());
  *inline_next = g->tensors[g->ltasks[i + 1].ops[0]].ndims == 2;
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_MOE_TOPK;
  if (*inline_next) st.flags |= MK_F_ONLY_MULTI;
  st.moe_logits = lg.ptr;
  st.ld_logits = (int)lg.strides[0];
  st.moe_topk_w = (float *)tw.ptr;
  st.ld_topk_w = (int)tw.strides[0];
  st.moe_routing = (int *)ri.ptr;
  st.ld_routing = (int)ri.strides[0];
  st.moe_mask = (int *)mk.ptr;
  st.num_experts = E;
  st.topk = topk;
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MOE_TOPK%s %s -> %s,%s experts=%d topk=%d", *inline_next ? "[multi-token only]" : "", lg.name.c_str(), tw.name.c_str(), ri.name.c_str(), E, topk));
  i++;
  return MK_OK;
}

// Per-expert linear [input, weight[E,N,K], routing_indices, mask, output[tokens,topk,N]]; input is [tokens, K] (every
// slot of a token sees the same row: W13) or [tokens, topk, K] (W2).  A directly following moe_silu_mul / moe_mul_sum_add
// over its output becomes the epilogue.
int lower_moe_linear(mk_graph *g, size_t &i, const MkStage *router) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 5) return fail(MK_EINVAL, "%s expects 5 operands", t.name.c_str());
  const Tensor &x = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &ri = g->tensors[t.ops[2]], &mk = g->tensors[t.ops[3]], &y = g->tensors[t.ops[4]];
  const int B = g->cfg.max_num_batched_tokens;
  if (w.ndims != 3 || w.dtype != MK_DT_BF16 || !w.ptr || w.strides[2] != 1 || w.strides[1] != w.dims[2] || w.strides[0] != w.dims[1] * w.dims[2])
    return fail(MK_EINVAL, "%s: weight '%s' must be a contiguous [experts, rows, k] bf16 tensor", t.name.c_str(), w.name.c_str());
  const int E = (int)w.dims[0], N = (int)w.dims[1], K = (int)w.dims[2];
  if (E > MK_MOE_MAX_EXPERTS) return fail(MK_EUNSUPPORTED, "%s: %d experts (max %d)", t.name.c_str(), E, MK_MOE_MAX_EXPERTS);
  if (K % 8 || K > 4096) return fail(MK_EUNSUPPORTED, "%s: k=%d must be a multiple of 8 and at most 4096", t.name.c_str(), K);
  if (ri.ndims != 2 || ri.dtype != MK_DT_I32 || ri.dims[0] != E || ri.dims[1] < B || ri.strides[1] != 1)
    return fail(MK_EINVAL, "%s: routing indices must be [experts, tokens] int32", t.name.c_str());
  if (mk.dtype != MK_DT_I32 || mk.elems() < (size_t)E + 1) return fail(MK_EINVAL, "%s: mask must hold experts+1 int32", t.name.c_str());
  if (!rows_contiguous_3d(y) || y.dtype != MK_DT_BF16 || y.dims[0] < B || y.dims[2] < N) return fail(MK_EINVAL, "%s: output must be [tokens, topk, %d] bf16", t.name.c_str(), N);
  const int topk = (int)y.dims[1];
  if (topk < 1 || topk > MK_MOE_MAX_TOPK) return fail(MK_EUNSUPPORTED, "%s: topk=%d (max %d)", t.name.c_str(), topk, MK_MOE_MAX_TOPK);
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_MOE_LINEAR;
  st.n = N;
  st.k = K;
  st.num_experts = E;
  st.topk = topk;
  st.w.nseg = 1;
  st.w.seg[0] = w.ptr;
  st.w.seg_rows[0] = st.w.group_rows = E * N;
  st.moe_routing = (int *)ri.ptr;
  st.ld_routing = (int)ri.strides[0];
  st.moe_mask = (int *)mk.ptr;
  st.in = x.ptr;
  if (x.dtype != MK_DT_BF16 || x.dims[0] < B) return fail(MK_EINVAL, "%s: input must be bf16 with at least %d token rows", t.name.c_str(), B);
  if (x.ndims == 2) {
    if (x.dims[1] != K || x.strides[1] != 1) return fail(MK_EINVAL, "%s: input must be [tokens, %d]", t.name.c_str(), K);
    st.ld_in = (int)x.strides[0];
  } else if (x.ndims == 3) {
    if (x.dims[1] != topk || x.dims[2] != K || x.strides[2] != 1) return fail(MK_EINVAL, "%s: input must be [tokens, %d, %d]", t.name.c_str(), topk, K);
    st.ld_in = (int)x.strides[0];
    st.ld_in_slot = (int)x.strides[1];
  } else {
    return fail(MK_EINVAL, "%s: input must be 2-D or 3-D", t.name.c_str());
  }
  if ((st.ld_in % 8) || (st.ld_in_slot % 8)) return fail(MK_EINVAL, "%s: input rows must be 16-byte aligned", t.name.c_str());
  st.out = y.ptr;
  st.ld_out = (int)y.strides[0];
  st.ld_out_slot = (int)y.strides[1];
  if (router) {
    st.flags |= MK_F_MOE_INLINE_TOPK;
    st.moe_logits = router->moe_logits;
    st.ld_logits = router->ld_logits;
    st.moe_topk_w = router->moe_topk_w;
    st.ld_topk_w = router->ld_topk_w;
    if (router->topk != topk || router->num_experts != E) return fail(MK_EINVAL, "%s: router has %d experts / top-%d, linear has %d / %d", t.name.c_str(), router->num_experts, router->topk, E, topk);
  }
  size_t consumed = 1;
  std::string extra;
  const Task *nx = i + 1 < g->ltasks.size() ? &g->ltasks[i + 1] : nullptr;
  if (nx && nx->name == "moe_silu_mul" && nx->ops.size() == 2 && nx->ops[0] == t.ops[4] && N % 2 == 0) {
    const Tensor &o = g->tensors[nx->ops[1]];
    if (!rows_contiguous_3d(o) || o.dtype != MK_DT_BF16 || o.dims[0] < B || o.dims[1] != topk || o.dims[2] != N / 2)
      return fail(MK_EINVAL, "moe_silu_mul: output must be [tokens, %d, %d] bf16", topk, N / 2);
    st.flags |= MK_F_SILU;
    st.out2 = o.ptr;
    st.ld_out2 = (int)o.strides[0];
    st.ld_out2_slot = (int)o.strides[1];
    consumed = 2;
    extra = "+silu -> " + o.name;
  } else if (nx && nx->name == "moe_mul_sum_add_mi300" && nx->ops.size() == 4 && nx->ops[0] == t.ops[4] && x.ndims == 3) {
    // fused for single-token iterations; the combine stage emitted by lower_moe_combine covers the others
    const Tensor &tw = g->tensors[nx->ops[1]], &r = g->tensors[nx->ops[2]], &o = g->tensors[nx->ops[3]];
    if (tw.ndims != 2 || tw.dtype != MK_DT_F32 || tw.dims[1] != topk || tw.strides[1] != 1 || r.ndims != 2 || o.ndims != 2 || r.dims[1] < N || o.dims[1] < N ||
        r.dtype != MK_DT_BF16 || o.dtype != MK_DT_BF16)
      return fail(MK_EINVAL, "moe_mul_sum_add_mi300: shapes do not match the expert outputs");
    st.flags |= MK_F_MOE_COMBINE;
    st.moe_topk_w = (float *)tw.ptr;
    st.ld_topk_w = (int)tw.strides[0];
    st.res = r.ptr;
    st.ld_res = (int)r.strides[0];
    st.out2 = o.ptr;
    st.ld_out2 = (int)o.strides[0];
    extra = "+combine(single token) -> " + o.name;
  }
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MOE_LINEAR%s %s x %s -> %s experts=%d topk=%d n=%d k=%d%s", router ? "+route(single token)" : "", x.name.c_str(), w.name.c_str(), y.name.c_str(), E,
                              topk, N, K, extra.c_str()));
  g->weight_bytes += (int64_t)topk * N * K * 2;  // bytes a single-token iteration streams
  i += consumed;
  return MK_OK;
}

// moe_mul_sum_add_mi300 [expert outputs [tokens,topk,n], routing weights [tokens,topk], residual, output]
int lower_moe_combine(mk_graph *g, size_t &i, bool fused_single) {
  const Task &t = g->ltasks[i];
  if (t.ops.size() != 4) return fail(MK_EINVAL, "%s expects 4 operands", t.name.c_str());
  const Tensor &x = g->tensors[t.ops[0]], &tw = g->tensors[t.ops[1]], &r = g->tensors[t.ops[2]], &o = g->tensors[t.ops[3]];
  const int B = g->cfg.max_num_batched_tokens;
  if (x.ndims != 3 || x.dtype != MK_DT_BF16 || x.strides[2] != 1 || x.dims[0] < B) return fail(MK_EINVAL, "%s: input must be [tokens, topk, n] bf16", t.name.c_str());
  const int topk = (int)x.dims[1], N = (int)x.dims[2];
  if (tw.ndims != 2 || tw.dtype != MK_DT_F32 || tw.dims[1] != topk || tw.strides[1] != 1 || tw.dims[0] < B) return fail(MK_EINVAL, "%s: weights must be [tokens, %d] fp32", t.name.c_str(), topk);
  if (r.ndims != 2 || o.ndims != 2 || r.dims[1] < N || o.dims[1] < N || r.dtype != MK_DT_BF16 || o.dtype != MK_DT_BF16 || r.dims[0] < B || o.dims[0] < B)
    return fail(MK_EINVAL, "%s: residual/output must be [tokens, >=%d] bf16", t.name.c_str(), N);
  MkStage st;
  memset(&st, 0, sizeof(st));
  st.op = MK_OP_MOE_COMBINE;
  if (fused_single) st.flags |= MK_F_ONLY_MULTI;
  st.n = N;
  st.topk = topk;
  st.in = x.ptr;
  st.ld_in = (int)x.strides[0];
  st.ld_in_slot = (int)x.strides[1];
  st.moe_topk_w = (float *)tw.ptr;
  st.ld_topk_w = (int)tw.strides[0];
  st.res = r.ptr;
  st.ld_res = (int)r.strides[0];
  st.out = o.ptr;
  st.ld_out = (int)o.strides[0];
  g->stages.push_back(st);
  g->stage_desc.push_back(fmt("MOE_COMBINE%s %s * %s + %s -> %s n=%d topk=%d", fused_single ? "[multi-token only]" : "", x.name.c_str(), tw.name.c_str(), r.name.c_str(), o.name.c_str(), N, topk));
  i++;
  return MK_OK;
}

int lower(mk_graph *g) {
  g->stages.clear();
  g->stage_desc.clear();
  g->stage_weight.clear();
  g->weight_bytes = 0;
  g->last_linear_task = g->last_linear_stage = -1;
  g->flex = FLEX_NONE;
  g->flex_items = g->flex_part = 0;
  g->mix = g->hyb = g->dual = false;
  g->state_ids = nullptr;
  const int B = g->cfg.max_num_batched_tokens;
  // The list that is lowered: the recorded tasks, with the composite ones spelt out as the tasks they stand for (the
  // task graph handed back to the caller keeps them as recorded).
  g->ltasks.clear();
  for (const Task &t : g->tasks) {
    if (t.name == "rmsnorm_linear") {
      // [input, norm weight, linear weight, output] (python/mirage/mpk/persistent_kernel.py:566-585): RMSNorm into a
      // library-owned row buffer, then a plain linear over it
      if (t.ops.size() != 4) return fail(MK_EINVAL, "rmsnorm_linear expects 4 operands");
      const Tensor &x = g->tensors[t.ops[0]];
      if (x.ndims != 2) return fail(MK_EINVAL, "rmsnorm_linear: input must be 2-D");
      const std::string nm = "rmsnorm_linear_norm_out_" + std::to_string(g->ltasks.size());
      int nid = -1;
      for (size_t k = 0; k < g->tensors.size(); k++)
        if (g->tensors[k].name == nm) nid = (int)k;
      if (nid < 0) {
        Tensor nt;
        nt.name = nm;
        nt.ndims = 2;
        nt.dtype = x.dtype;
        nt.kind = T_OWNED;
        nt.dims[0] = x.dims[0];
        nt.dims[1] = x.dims[1];
        nt.strides[0] = x.dims[1];
        nt.strides[1] = 1;
        void *p = nullptr;
        int rc = dev_alloc(g, &p, (size_t)x.dims[0] * x.dims[1] * dtype_size(x.dtype));
        if (rc) return rc;
        nt.ptr = p;
        g->tensors.push_back(nt);
        nid = (int)g->tensors.size() - 1;
      }
      Task n = t, l = t;
      n.name = "rmsnorm";
      n.ops = {t.ops[0], t.ops[1], nid};
      n.maps = {t.maps[0], t.maps[1], t.maps[0]};
      n.forloop = {t.forloop[0], t.forloop[1], t.forloop[0]};
      n.params.clear();
      l.name = "linear";
      l.ops = {nid, t.ops[2], t.ops[3]};
      l.maps = {t.maps[0], t.maps[2], t.maps[3]};
      l.forloop = {t.forloop[0], t.forloop[2], t.forloop[3]};
      l.params.clear();
      g->ltasks.push_back(n);
      g->ltasks.push_back(l);
    } else {
      g->ltasks.push_back(t);
    }
  }
  size_t i = 0;
  while (i < g->ltasks.size()) {
    const Task &t = g->ltasks[i];
    bool res, silu;
    int extra;
    if (t.name == "embedding") {
      if (t.ops.size() != 3) return fail(MK_EINVAL, "embedding expects 3 operands");
      const Tensor &ids = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &o = g->tensors[t.ops[2]];
      if (ids.dtype != MK_DT_I64) return fail(MK_EINVAL, "embedding ids must be int64");
      if (w.ndims != 2 || o.ndims != 2 || w.dims[1] != o.dims[1] || w.dims[1] % 8 || w.dtype != MK_DT_BF16) return fail(MK_EINVAL, "embedding shapes mismatch");
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = MK_OP_EMBED;
      st.k = (int)w.dims[1];
      st.in = ids.ptr;
      st.out = o.ptr;
      st.ld_out = (int)o.strides[0];
      st.w.nseg = 1;
      st.w.seg[0] = w.ptr;
      if (!t.params.empty() && t.params[0] == 0) st.flags |= MK_F_EMBED_FROM_TOKENS;
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("EMBED %s[%s] -> %s k=%d", w.name.c_str(), ids.name.c_str(), o.name.c_str(), st.k));
      i++;
    } else if (is_norm(t.name)) {
      if (t.ops.size() != 3) return fail(MK_EINVAL, "%s expects 3 operands", t.name.c_str());
      if (i + 1 < g->ltasks.size() && linear_kind(g->ltasks[i + 1].name, &res, &silu, &extra) && g->ltasks[i + 1].ops[0] == t.ops[2]) {
        int rc = lower_linear(g, i);
        if (rc) return rc;
      } else {
        const Tensor &x = g->tensors[t.ops[0]], &w = g->tensors[t.ops[1]], &o = g->tensors[t.ops[2]];
        if (x.ndims != 2 || o.ndims != 2 || x.dims[1] != o.dims[1] || w.elems() != (size_t)x.dims[1] || x.dims[1] % 8)
          return fail(MK_EINVAL, "%s shapes mismatch", t.name.c_str());
        MkStage st;
        memset(&st, 0, sizeof(st));
        st.op = MK_OP_NORM;
        st.k = (int)x.dims[1];
        st.eps = g->cfg.rms_eps;
        st.in = x.ptr;
        st.ld_in = (int)x.strides[0];
        st.norm_w = w.ptr;
        st.out = o.ptr;
        st.ld_out = (int)o.strides[0];
        g->stages.push_back(st);
        g->stage_desc.push_back(fmt("NORM %s -> %s k=%d", x.name.c_str(), o.name.c_str(), st.k));
        i++;
      }
    } else if (linear_kind(t.name, &res, &silu, &extra)) {
      int rc = lower_linear(g, i);
      if (rc) return rc;
    } else if (t.name == "silu_mul_linear_with_residual") {
      int rc = lower_silu_mul_linear(g, i);
      if (rc) return rc;
    } else if (t.name == "silu_mul") {
      if (t.ops.size() != 2) return fail(MK_EINVAL, "silu_mul expects 2 operands");
      const Tensor &x = g->tensors[t.ops[0]], &o = g->tensors[t.ops[1]];
      const int groups = t.grid[0] * t.grid[1] * t.grid[2];
      if (x.ndims != 2 || o.ndims != 2 || x.dims[1] != 2 * o.dims[1] || groups <= 0 || o.dims[1] % groups) return fail(MK_EINVAL, "silu_mul shapes mismatch");
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = MK_OP_SILU_MUL;
      st.n = (int)o.dims[1];
      st.silu_half = (int)(o.dims[1] / groups);
      st.groups = groups;
      st.in = x.ptr;
      st.ld_in = (int)x.strides[0];
      st.out = o.ptr;
      st.ld_out = (int)o.strides[0];
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("SILU_MUL %s -> %s n=%d half=%d", x.name.c_str(), o.name.c_str(), st.n, st.silu_half));
      i++;
    } else if (t.name == "gang_attn_split_kv_mi300" || t.name == "kv_cache_update_mi300" || t.name == "paged_attention" ||
               t.name == "paged_attention_split_kv_mi300" || t.name == "attention" || t.name == "single_batch_extend_attention") {
      int rc = lower_attention(g, i);
      if (rc) return rc;
    } else if (t.name == "embedding_scaled") {
      int rc = lower_embedding_scaled(g, i);
      if (rc) return rc;
    } else if (t.name == "residual_rmsnorm") {
      int rc = lower_residual_rmsnorm(g, i);
      if (rc) return rc;
    } else if (t.name == "flex_attention") {
      int rc = lower_flex_attention(g, i);
      if (rc) return rc;
    } else if (t.name == "residual_prenorm") {
      int rc = lower_residual_prenorm(g, i);
      if (rc) return rc;
    } else if (t.name == "latent_prep") {
      int rc = lower_latent_prep(g, i);
      if (rc) return rc;
    } else if (t.name == "head_linear") {
      int rc = lower_head_linear(g, i);
      if (rc) return rc;
    } else if (t.name == "latent_attention") {
      int rc = lower_latent_attention(g, i);
      if (rc) return rc;
    } else if (t.name == "general_delta") {
      int rc = lower_general_delta(g, i);
      if (rc) return rc;
    } else if (t.name == "short_conv") {
      int rc = lower_short_conv(g, i);
      if (rc) return rc;
    } else if (t.name == "ring_conv") {
      int rc = lower_ring_conv(g, i, nullptr, nullptr);
      if (rc) return rc;
    } else if (t.name == "dual_scan") {
      int rc = lower_dual_scan(g, i);
      if (rc) return rc;
    } else if (t.name == "gelu_mul") {
      return fail(MK_EUNSUPPORTED, "gelu_mul follows the linear that writes its input");
    } else if (t.name == "scan_step") {
      int rc = lower_scan_step(g, i);
      if (rc) return rc;
    } else if (t.name == "selective_scan") {
      int rc = lower_selective_scan(g, i);
      if (rc) return rc;
    } else if (t.name == "expert_route") {
      int rc = lower_expert_route(g, i);
      if (rc) return rc;
    } else if (t.name == "expert_linear") {
      int rc = lower_expert_linear(g, i);
      if (rc) return rc;
    } else if (t.name == "moe_topk_softmax_mi300") {
      bool inline_next = false;
      int rc = lower_moe_topk(g, i, &inline_next);
      if (rc) return rc;
      const MkStage router = g->stages.back();
      rc = lower_moe_linear(g, i, inline_next ? &router : nullptr);
      if (rc) return rc;
    } else if (is_moe_linear(t.name)) {
      int rc = lower_moe_linear(g, i, nullptr);
      if (rc) return rc;
    } else if (t.name == "moe_mul_sum_add_mi300") {
      const bool fused = !g->stages.empty() && g->stages.back().op == MK_OP_MOE_LINEAR && (g->stages.back().flags & MK_F_MOE_COMBINE) &&
                         g->stages.back().out == g->tensors[t.ops.empty() ? 0 : t.ops[0]].ptr;
      int rc = lower_moe_combine(g, i, fused);
      if (rc) return rc;
    } else if (t.name == "moe_silu_mul") {
      if (t.ops.size() != 2) return fail(MK_EINVAL, "moe_silu_mul expects 2 operands");
      const Tensor &x = g->tensors[t.ops[0]], &o = g->tensors[t.ops[1]];
      if (!rows_contiguous_3d(x) || !rows_contiguous_3d(o) || x.dims[2] != 2 * o.dims[2] || x.dims[1] != o.dims[1] || x.dtype != MK_DT_BF16 || o.dtype != MK_DT_BF16)
        return fail(MK_EINVAL, "moe_silu_mul shapes mismatch");
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = MK_OP_SILU_MUL;
      st.n = (int)o.dims[2];
      st.silu_half = st.n;  // [gate ; up] halves of every (token, slot) row
      st.groups = 1;
      st.topk = (int)x.dims[1];
      st.in = x.ptr;
      st.ld_in = (int)x.strides[1];
      st.out = o.ptr;
      st.ld_out = (int)o.strides[1];
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("SILU_MUL(moe) %s -> %s n=%d rows/token=%d", x.name.c_str(), o.name.c_str(), st.n, st.topk));
      i++;
    } else if (t.name == "identity") {
      // [input, output], same shape (python/mirage/mpk/persistent_kernel.py:2153-2172; tasks/ampere/identity.cuh:24-37)
      if (t.ops.size() != 2) return fail(MK_EINVAL, "identity expects 2 operands");
      const Tensor &x = g->tensors[t.ops[0]], &o = g->tensors[t.ops[1]];
      if (x.ndims != o.ndims || x.ndims < 2 || x.dtype != o.dtype || x.kind == T_SHUFFLED || o.kind == T_SHUFFLED) return fail(MK_EINVAL, "identity: input and output must be stored tensors of one shape and dtype");
      int64_t inner = 1;
      for (int d = 0; d < x.ndims; d++) {
        if (x.dims[d] != o.dims[d] || x.strides[d] != o.strides[d]) return fail(MK_EINVAL, "identity: input and output shapes differ");
        if (d) inner *= x.dims[d];
      }
      if (x.strides[0] != inner) return fail(MK_EINVAL, "identity: rows must be contiguous");
      if (x.dims[0] < B) return fail(MK_EINVAL, "identity: tensors need at least max_num_batched_tokens=%d rows", B);
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = MK_OP_COPY;
      st.n = (int)(inner * (int64_t)dtype_size(x.dtype) / 2);  // 16-bit units per token row
      st.in = x.ptr;
      st.out = o.ptr;
      st.ld_in = st.ld_out = st.n;
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("COPY %s -> %s units=%d", x.name.c_str(), o.name.c_str(), st.n));
      i++;
    } else if (t.name == "argmax") {
      // [logits, output] in one task (python/mirage/mpk/persistent_kernel.py:2195-2205): the same two stages as the
      // partial + reduce pair, over library-owned partials
      if (t.ops.size() != 2) return fail(MK_EINVAL, "argmax expects 2 operands");
      const Tensor &x = g->tensors[t.ops[0]], &o = g->tensors[t.ops[1]];
      if (x.ndims != 2 || (x.dtype != MK_DT_BF16 && x.dtype != MK_DT_F32) || o.dtype != MK_DT_I64) return fail(MK_EINVAL, "argmax: logits must be 2-D bf16 or fp32 and the output int64");
      void *pv = nullptr, *pi = nullptr;
      int rc = dev_alloc(g, &pv, sizeof(float) * (size_t)B * g->G);
      if (rc) return rc;
      rc = dev_alloc(g, &pi, sizeof(int) * (size_t)B * g->G);
      if (rc) return rc;
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = x.dtype == MK_DT_F32 ? MK_OP_FX_ARGMAX_F32 : MK_OP_ARGMAX_PARTIAL;
      st.n = (int)x.dims[1];
      st.in = x.ptr;
      st.ld_in = (int)x.strides[0];
      st.aux0 = pv;
      st.aux1 = pi;
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("ARGMAX_PARTIAL %s n=%d", x.name.c_str(), st.n));
      MkStage sr;
      memset(&sr, 0, sizeof(sr));
      sr.op = MK_OP_ARGMAX_REDUCE;
      sr.aux0 = pv;
      sr.aux1 = pi;
      sr.out = o.ptr;
      g->stages.push_back(sr);
      g->stage_desc.push_back(fmt("ARGMAX_REDUCE -> %s", o.name.c_str()));
      i++;
    } else if (t.name == "argmax_partial") {
      if (t.ops.size() != 3) return fail(MK_EINVAL, "argmax_partial expects 3 operands");
      if (i + 1 >= g->ltasks.size() || g->ltasks[i + 1].name != "argmax_reduce" || g->ltasks[i + 1].ops.size() != 3)
        return fail(MK_EUNSUPPORTED, "argmax_partial must be followed by argmax_reduce");
      const Tensor &x = g->tensors[t.ops[0]], &o = g->tensors[g->ltasks[i + 1].ops[2]];
      if (x.ndims != 2 || (x.dtype != MK_DT_BF16 && x.dtype != MK_DT_F32) || o.dtype != MK_DT_I64) return fail(MK_EINVAL, "argmax: logits must be 2-D bf16 or fp32 and the output int64");
      void *pv = nullptr, *pi = nullptr;
      int rc = dev_alloc(g, &pv, sizeof(float) * (size_t)B * g->G);
      if (rc) return rc;
      rc = dev_alloc(g, &pi, sizeof(int) * (size_t)B * g->G);
      if (rc) return rc;
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = x.dtype == MK_DT_F32 ? MK_OP_FX_ARGMAX_F32 : MK_OP_ARGMAX_PARTIAL;
      st.n = (int)x.dims[1];
      st.in = x.ptr;
      st.ld_in = (int)x.strides[0];
      st.aux0 = pv;
      st.aux1 = pi;
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("ARGMAX_PARTIAL %s n=%d", x.name.c_str(), st.n));
      MkStage sr;
      memset(&sr, 0, sizeof(sr));
      sr.op = MK_OP_ARGMAX_REDUCE;
      sr.aux0 = pv;
      sr.aux1 = pi;
      sr.out = o.ptr;
      g->stages.push_back(sr);
      g->stage_desc.push_back(fmt("ARGMAX_REDUCE -> %s", o.name.c_str()));
      i += 2;
    } else if (t.name == "find_ngram_partial") {
      // (tokens, partial) + [ngram size]; src/kernel/task_register.cc:1689-1719
      if (t.ops.size() != 2 || t.params.size() != 1) return fail(MK_EINVAL, "find_ngram_partial expects (tokens, partial results) and the n-gram size");
      const Tensor &tk = g->tensors[t.ops[0]], &po = g->tensors[t.ops[1]];
      if (tk.ptr != (void *)g->cfg.tokens) return fail(MK_EINVAL, "find_ngram_partial searches the `tokens` meta tensor: attach that tensor as its input");
      if (po.ndims != 2 || po.dtype != MK_DT_I64 || po.dims[0] < g->cfg.max_num_batched_requests || po.dims[1] < 1)
        return fail(MK_EINVAL, "find_ngram_partial: the partial results are an int64 [batch slots >= %d, tasks] tensor", g->cfg.max_num_batched_requests);
      if (t.params[0] < 1 || t.params[0] > 16) return fail(MK_EINVAL, "find_ngram_partial: n-gram size %d outside [1, 16]", t.params[0]);
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = MK_OP_NGRAM_PARTIAL;
      st.n = (int)po.dims[1];
      st.k = t.params[0];
      st.out = po.ptr;
      st.ld_out = (int)po.strides[0];
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("NGRAM_PARTIAL %s -> %s ngram=%d tasks=%d", tk.name.c_str(), po.name.c_str(), st.k, st.n));
      i++;
    } else if (t.name == "find_ngram_global") {
      // (partial, tokens, spec tokens) + [ngram size, spec length]; task_register.cc:1721-1754
      if (t.ops.size() != 3 || t.params.size() != 2) return fail(MK_EINVAL, "find_ngram_global expects (partial results, tokens, spec tokens) and (n-gram size, spec length)");
      const Tensor &pi = g->tensors[t.ops[0]], &tk = g->tensors[t.ops[1]], &so = g->tensors[t.ops[2]];
      if (tk.ptr != (void *)g->cfg.tokens) return fail(MK_EINVAL, "find_ngram_global reads the `tokens` meta tensor: attach that tensor as its input");
      if (pi.ndims != 2 || pi.dtype != MK_DT_I64 || pi.dims[0] < g->cfg.max_num_batched_requests) return fail(MK_EINVAL, "find_ngram_global: bad partial-result tensor");
      if (so.dtype != MK_DT_I64 || (long long)so.elems() < B) return fail(MK_EINVAL, "find_ngram_global: the spec-token tensor holds one int64 id per token row of an iteration (>= %d)", B);
      const int spec_len = t.params[1];
      if (spec_len < 1) return fail(MK_EINVAL, "find_ngram_global: spec length %d < 1", spec_len);
      if (g->cfg.mode != MK_MODE_OFFLINE) return fail(MK_EUNSUPPORTED, "speculative decoding needs the offline scheduler (mode offline): it sizes the token groups of decoding requests");
      if (B < spec_len + 1) return fail(MK_EINVAL, "speculative decoding with %d guesses needs max_num_batched_tokens >= %d", spec_len, spec_len + 1);
      if ((g->cfg.max_tokens_per_request > 0 ? g->cfg.max_tokens_per_request : 8) < spec_len + 1)
        return fail(MK_EINVAL, "speculative decoding with %d guesses needs max_tokens_per_request >= %d (a decoding request brings that many rows)", spec_len, spec_len + 1);
      if (g->spec_len && g->spec_len != spec_len) return fail(MK_EINVAL, "two find_ngram_global tasks with different spec lengths");
      g->spec_len = spec_len;
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = MK_OP_NGRAM_GLOBAL;
      st.n = (int)pi.dims[1];
      st.k = t.params[0];
      st.topk = spec_len;
      st.in = pi.ptr;
      st.ld_in = (int)pi.strides[0];
      st.out = so.ptr;
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("NGRAM_GLOBAL %s, %s -> %s ngram=%d spec=%d", pi.name.c_str(), tk.name.c_str(), so.name.c_str(), st.k, spec_len));
      i++;
    } else if (t.name == "target_verify_greedy") {
      // (spec tokens, target tokens, accepted length); task_register.cc:1756-1784
      if (t.ops.size() != 3) return fail(MK_EINVAL, "target_verify_greedy expects (spec tokens, target tokens, output)");
      const Tensor &sp = g->tensors[t.ops[0]], &tg = g->tensors[t.ops[1]], &vo = g->tensors[t.ops[2]];
      if (sp.dtype != MK_DT_I64 || tg.dtype != MK_DT_I64 || vo.dtype != MK_DT_I64 || (long long)sp.elems() < B || (long long)tg.elems() < B || vo.elems() < 1)
        return fail(MK_EINVAL, "target_verify_greedy: spec and target tokens hold one int64 id per token row (>= %d), the output one int64", B);
      if (!g->cfg.num_new_tokens) return fail(MK_EINVAL, "target_verify_greedy writes the num_new_tokens meta tensor: it must be given");
      if (!g->spec_len) return fail(MK_EINVAL, "target_verify_greedy without a find_ngram_global task before it");
      MkStage st;
      memset(&st, 0, sizeof(st));
      st.op = MK_OP_VERIFY;
      st.in = sp.ptr;
      st.aux0 = tg.ptr;
      st.out = vo.ptr;
      g->stages.push_back(st);
      g->stage_desc.push_back(fmt("VERIFY %s vs %s -> num_new_tokens, %s", sp.name.c_str(), tg.name.c_str(), vo.name.c_str()));
      i++;
    } else if (t.name == "paged_attention_split_kv_merge_mi300" || t.name == "paged_attention_ck_fmha_merge_mi300" || t.name == "gang_attn_merge_mi300" ||
               t.name == "splitk_reduce_mi300") {
      return fail(MK_EUNSUPPORTED, "task '%s' must directly follow the split task whose partial results it combines", t.name.c_str());
    } else {
      return fail(MK_EUNSUPPORTED, "task '%s' has no MI355X lowering", t.name.c_str());
    }
  }
  if (g->spec_len && g->state_ids) return fail(MK_EUNSUPPORTED, "speculative decoding with a recurrence: rows of rejected guesses cannot be taken back out of its state");
  g->stage_weight.resize(g->stages.size(), -1);
  for (size_t s = 0; s < g->stages.size(); s++) {
    const int op = g->stages[s].op;
    const bool f32_op = op == MK_OP_LINEAR_F32 || op == MK_OP_FX_ARGMAX_F32;
    const bool fixed_op = op == MK_OP_EMBED || op == MK_OP_NORM || op == MK_OP_ATTN || op == MK_OP_SILU_MUL || op == MK_OP_MOE_TOPK || op == MK_OP_MOE_LINEAR || op == MK_OP_MOE_COMBINE;
    const bool ok = g->flex == FLEX_NONE ? !f32_op : g->flex == FLEX_BF16 ? !f32_op && !fixed_op : !fixed_op && op != MK_OP_LINEAR && op != MK_OP_ARGMAX_PARTIAL;
    const bool not_dual = (op >= MK_OP_MX_LATENT_PREP && op <= MK_OP_MX_DELTA_OUT && op != MK_OP_MX_HEAD_LINEAR) || (op >= MK_OP_HY_CONV && op <= MK_OP_HY_SCAN);
    if (!ok || (g->dual && not_dual)) return fail(MK_EUNSUPPORTED, "stage %zu (%s) cannot run in one graph with the others", s, g->stage_desc[s].c_str());
  }
  for (auto &st : g->stages) {  // the task type a stage is shown as in a profiler trace (runtime_header.h:91-188)
    switch (st.op) {
      case MK_OP_EMBED: st.prof_event = 101; break;
      case MK_OP_NORM: st.prof_event = 119; break;
      case MK_OP_LINEAR: st.prof_event = (st.flags & MK_F_NORM) ? 102 : ((st.flags & MK_F_RES) ? 108 : 120); break;
      case MK_OP_SILU_MUL: st.prof_event = 118; break;
      case MK_OP_ATTN: st.prof_event = 116; break;
      case MK_OP_ARGMAX_PARTIAL: st.prof_event = 110; break;
      case MK_OP_ARGMAX_REDUCE: st.prof_event = 111; break;
      case MK_OP_MOE_TOPK: st.prof_event = 172; break;
      case MK_OP_MOE_LINEAR: st.prof_event = (st.flags & MK_F_MOE_COMBINE) || st.ld_in_slot ? 171 : 170; break;
      case MK_OP_MOE_COMBINE: st.prof_event = 173; break;
      case MK_OP_FX_EMBED: st.prof_event = 101; break;
      case MK_OP_FX_ADDNORM: st.prof_event = 119; break;
      case MK_OP_FX_PREP:
      case MK_OP_FX_ATTN: st.prof_event = 116; break;
      case MK_OP_LINEAR_F32:
      case MK_OP_MX_HEAD_LINEAR: st.prof_event = 120; break;
      case MK_OP_MX_PRENORM: st.prof_event = 119; break;
      case MK_OP_MX_LATENT_PREP:
      case MK_OP_MX_LATENT_ATTN:
      case MK_OP_MX_LATENT_MERGE:
      case MK_OP_MX_DECAY:
      case MK_OP_MX_DELTA:
      case MK_OP_MX_DELTA_OUT:
      case MK_OP_HY_CONV:
      case MK_OP_HY_SCAN:
      case MK_OP_DU_CONV:
      case MK_OP_DU_SCAN: st.prof_event = 116; break;
      case MK_OP_HY_STEP: st.prof_event = 120; break;
      case MK_OP_HY_ROUTE: st.prof_event = 172; break;
      case MK_OP_HY_EXPERTS: st.prof_event = (st.flags & MK_F_SILU) ? 170 : 171; break;
      case MK_OP_FX_ARGMAX_F32: st.prof_event = 110; break;
      case MK_OP_NGRAM_PARTIAL: st.prof_event = 112; break;
      case MK_OP_NGRAM_GLOBAL: st.prof_event = 113; break;
      case MK_OP_VERIFY: st.prof_event = 114; break;
      default: st.prof_event = 121; break;
    }
  }
  g->program_text.clear();
  for (size_t s = 0; s < g->stage_desc.size(); s++) g->program_text += fmt("%3zu ", s) + g->stage_desc[s] + "\n";
  return MK_OK;
}

// ---- reference-shaped task graph (JSON) ------------------------------------------------------
// The task / event graph the reference's Graph::generate_task_graph builds for the recorded operators
// (src/kernel/runtime.cc:164-612, printed by print_task_graph :948-1437), re-derived:
//   * task 0 = TERMINATE, task 1 = BEGIN_TASK_GRAPH; event 0 = TERMINATION, event 1 = LAUNCH_DEPENDENT_TASKS over
//     [2, #tasks); the last event = END_OF_TASK_GRAPH, triggered by every task of the last operator (:176-182,580-595);
//   * the first operator's tasks follow in (bid.x, bid.y, bid.z) order and are the "first_tasks" (:499-513);
//   * between operators i and i+1 the dependency is carried by ONE tensor -- the last (consumer input, producer output)
//     pair naming the same tensor (:519-531); along each of its dims the number of events is gcd(producer partition,
//     consumer partition) (:533-557); an event holds the consumer blocks whose index along the mapped grid axis falls
//     into its slice, in bid order, and is triggered by the producer blocks of the matching slice (:53-140).  Consumer
//     tasks are therefore stored event by event, not in plain bid order;
//   * every launch event ends as EVENT_EMPTY, its tasks carrying `dependent_event` (:593-611; the LAUNCH_TASKS /
//     LAUNCH_MASSIVE_TASKS distinction of :102-105 does not survive that rewrite); tasks without a dependency and the
//     two bookkeeping tasks carry EVENT_INVALID_ID.
// The six metadata keys are views of one 8-byte union that starts as all ones (runtime_header.h:223-256) and receives
// the writes of runtime.cc:365-452 in that order -- including the request_id = bid.x every task gets through the
// always-true term at :380.  Two operators that share no tensor (the reference asserts) get one event from all
// producer blocks to all consumer blocks.
struct RefTask {
  int op_index;
  int bid[3];
  unsigned long long trigger_event, dependent_event;
};
struct RefEvent {
  int type, num_triggers, first_task, last_task;
};
static const unsigned long long REF_EVENT_INVALID = 0x7ffffffffffffffeull;

int task_type_id(const std::string &n) {
  // runtime_header.h:91-188 task ids for the tasks this library lowers
  static const std::map<std::string, int> ids = {
      {"embedding", 101},       {"rmsnorm", 119},          {"gang_rmsnorm_mi300", 143}, {"linear", 120},
      {"linear_with_residual", 108}, {"silu_mul", 118},    {"argmax_partial", 110},     {"argmax_reduce", 111},
      {"splitk_linear_res_atomic_mi300", 133}, {"gang_linear_mi300", 136}, {"gang_linear_res_mi300", 137},
      {"gang_attn_split_kv_mi300", 138}, {"kv_cache_update_mi300", 140}, {"paged_attention_ck_fmha_split_kv_mi300", 141},
      {"gang_linear_silu_mi300", 142}, {"linear_silu_mi300", 182}, {"splitk_linear_mi300", 129}, {"gang_splitk_linear_res_mi300", 144},
      {"gang_linear_n_tiling_mi300", 147}, {"gang_linear_res_n_tiling_mi300", 148}, {"gang_linear_msplit_mi300", 183},
      {"gang_linear_res_msplit_mi300", 184}, {"moe_w13_linear_mi300", 170}, {"moe_w2_linear_mi300", 171}, {"moe_topk_softmax_mi300", 172},
      {"moe_mul_sum_add_mi300", 173}, {"gang_moe_w13_linear_mi300", 174}, {"gang_moe_w2_linear_mi300", 175}, {"moe_silu_mul", 118},
      {"paged_attention", 116}, {"paged_attention_split_kv_mi300", 130}, {"paged_attention_split_kv_merge_mi300", 131},
      {"paged_attention_ck_fmha_merge_mi300", 131}, {"gang_attn_merge_mi300", 139}, {"splitk_reduce_mi300", 132},
      {"silu_mul_linear_with_residual", 105}, {"rmsnorm_linear", 102}, {"identity", 121}, {"argmax", 109}, {"attention", 103},
      {"find_ngram_partial", 112}, {"find_ngram_global", 113}, {"target_verify_greedy", 114}, {"single_batch_extend_attention", 115},
      {"embedding_scaled", 101}, {"residual_rmsnorm", 119}, {"flex_attention", 116},
      {"residual_prenorm", 119}, {"latent_prep", 116}, {"head_linear", 120}, {"latent_attention", 116}, {"general_delta", 116},
      {"relu_squared", 118}, {"short_conv", 116}, {"scan_step", 120}, {"selective_scan", 116}, {"expert_route", 172}, {"expert_linear", 170}, {"ring_conv", 116},
      {"dual_scan", 116}, {"gelu_mul", 118}};
  auto it = ids.find(n);
  return it == ids.end() ? 0 : it->second;
}

// which param of a gang task is its tiles-per-XCD count (src/kernel/graph.cc:584-675,825-838); -1: not a gang task
int gang_tiles_param(const std::string &n) {
  if (n == "gang_linear_mi300" || n == "gang_linear_n_tiling_mi300" || n == "gang_linear_res_mi300" || n == "gang_linear_res_n_tiling_mi300" ||
      n == "gang_linear_silu_mi300")
    return 4;
  if (n == "gang_linear_msplit_mi300" || n == "gang_linear_res_msplit_mi300") return 3;
  if (n == "gang_rmsnorm_mi300") return 0;
  if (n == "gang_attn_split_kv_mi300") return 7;
  if (n == "gang_attn_merge_mi300") return 5;
  if (n == "gang_moe_w13_linear_mi300" || n == "gang_moe_w2_linear_mi300") return 2;
  if (n == "gang_splitk_linear_res_mi300") return -2;  // params[2] * params[3]
  return -1;
}

// The 8-byte metadata union of a task (runtime_header.h:238-256), little endian: bytes 0-1 request_id / n_tile_start,
// bytes 2-3 kv_idx / n_tile_count, bytes 0-3 expert_offset, bytes 4-7 merge_task_offset / _linear_reserved.
unsigned long long ref_task_metadata(const Task &t, const int bid[3]) {
  unsigned long long m = ~0ull;
  auto set16 = [&](int at, unsigned v) { m = (m & ~(0xffffull << (8 * at))) | ((unsigned long long)(v & 0xffffu) << (8 * at)); };
  auto set32 = [&](int at, unsigned v) { m = (m & ~(0xffffffffull << (8 * at))) | ((unsigned long long)v << (8 * at)); };
  const int type = task_type_id(t.name);
  set16(0, (unsigned)bid[0]);  // request_id: written for every task (runtime.cc:380 is a bare enumerator in an || chain)
  if (type == 170 || type == 171 || type == 182) set32(0, (unsigned)((bid[1] << 16) | (bid[0] & 0xFFFF)));
  const int gp = gang_tiles_param(t.name);
  if (gp != -1) {
    int tiles = 0;
    if (gp == -2) tiles = t.params.size() > 3 ? t.params[2] * t.params[3] : 0;
    else tiles = (int)t.params.size() > gp ? t.params[gp] : 0;
    set16(2, (unsigned)tiles);
    if (type == 183 || type == 184) {
      set16(0, 0);
      set32(4, (unsigned)bid[0]);
    } else if (type == 138 || type == 139) {
      set16(0, (unsigned)(bid[0] * tiles));
    } else {
      set16(0, 0);
    }
  }
  if (type == 130 || type == 131 || type == 141) {
    set16(2, (unsigned)bid[2]);
    set32(4, (unsigned)bid[1]);
  }
  return m;
}

// partition of a tensor along each of its dims by one operand's grid mapping (later axes override earlier ones)
void partition_of(const Task &t, int operand, int part[4]) {
  for (int d = 0; d < 4; d++) part[d] = 1;
  for (int a = 0; a < 3; a++) {
    const int d = t.maps[operand][a];
    if (d >= 0 && d < 4) part[d] = t.grid[a];
  }
}

int build_task_graph_json(mk_graph *g) {
  std::vector<RefTask> tasks;
  std::vector<RefEvent> events;
  tasks.push_back({-1, {0, 0, 0}, REF_EVENT_INVALID, REF_EVENT_INVALID});  // TERMINATE
  tasks.push_back({-1, {0, 0, 0}, 1, REF_EVENT_INVALID});                  // BEGIN_TASK_GRAPH triggers event 1
  events.push_back({911 /*EVENT_TERMINATION*/, 1, 0, 0});
  events.push_back({903 /*EVENT_LAUNCH_DEPENDENT_TASKS*/, 1, 2, 0});
  std::vector<int> first_tasks;
  std::map<std::array<int, 3>, int> pre_map, cur_map;  // bid -> task index, of the previous / current operator
  for (size_t oi = 0; oi < g->tasks.size(); oi++) {
    const Task &c = g->tasks[oi];
    cur_map.clear();
    if (oi == 0) {
      for (int x = 0; x < c.grid[0]; x++)
        for (int y = 0; y < c.grid[1]; y++)
          for (int z = 0; z < c.grid[2]; z++) {
            cur_map[{x, y, z}] = (int)tasks.size();
            first_tasks.push_back((int)tasks.size());
            tasks.push_back({(int)oi, {x, y, z}, REF_EVENT_INVALID, REF_EVENT_INVALID});
          }
      pre_map = cur_map;
      continue;
    }
    const Task &p = g->tasks[oi - 1];
    // the tensor that carries the dependency: the last (consumer input, producer output) pair naming the same tensor
    const int c_in = (int)c.ops.size() - num_outputs(c), p_in = (int)p.ops.size() - num_outputs(p);
    int co = -1, po = -1;
    for (int a = 0; a < c_in; a++)
      for (int b = p_in; b < (int)p.ops.size(); b++)
        if (c.ops[a] >= 0 && c.ops[a] == p.ops[b]) {
          co = a;
          po = b;
        }
    int ev_dims[4] = {1, 1, 1, 1};
    std::array<int, 3> in_map = {-1, -1, -1}, out_map = {-1, -1, -1};
    if (co >= 0) {
      int pp[4], cp[4];
      in_map = c.maps[co];
      out_map = p.maps[po];
      partition_of(c, co, cp);
      partition_of(p, po, pp);
      for (int d = 0; d < 4; d++) ev_dims[d] = std::gcd(pp[d], cp[d]);
    }
    // depth-first over the tensor's dims: each combination of slices is one event
    int idx[4];
    for (idx[0] = 0; idx[0] < ev_dims[0]; idx[0]++)
      for (idx[1] = 0; idx[1] < ev_dims[1]; idx[1]++)
        for (idx[2] = 0; idx[2] < ev_dims[2]; idx[2]++)
          for (idx[3] = 0; idx[3] < ev_dims[3]; idx[3]++) {
            int clo[3] = {0, 0, 0}, chi[3] = {c.grid[0], c.grid[1], c.grid[2]}, plo[3] = {0, 0, 0}, phi[3] = {p.grid[0], p.grid[1], p.grid[2]};
            for (int d = 0; d < 4; d++)
              for (int a = 0; a < 3; a++) {
                if (in_map[a] == d) {
                  const int f = c.grid[a] / ev_dims[d];
                  clo[a] = idx[d] * f;
                  chi[a] = (idx[d] + 1) * f;
                }
                if (out_map[a] == d) {
                  const int f = p.grid[a] / ev_dims[d];
                  plo[a] = idx[d] * f;
                  phi[a] = (idx[d] + 1) * f;
                }
              }
            const int ev = (int)events.size();
            RefEvent e = {900 /*EVENT_EMPTY: its tasks carry dependent_event*/, 0, (int)tasks.size(), 0};
            for (int x = clo[0]; x < chi[0]; x++)
              for (int y = clo[1]; y < chi[1]; y++)
                for (int z = clo[2]; z < chi[2]; z++) {
                  cur_map[{x, y, z}] = (int)tasks.size();
                  tasks.push_back({(int)oi, {x, y, z}, REF_EVENT_INVALID, (unsigned long long)ev});
                }
            e.last_task = (int)tasks.size();
            for (int x = plo[0]; x < phi[0]; x++)
              for (int y = plo[1]; y < phi[1]; y++)
                for (int z = plo[2]; z < phi[2]; z++) {
                  auto it = pre_map.find({x, y, z});
                  if (it == pre_map.end()) return fail(MK_EINVAL, "task graph: producer block (%d,%d,%d) of '%s' has no task", x, y, z, p.name.c_str());
                  tasks[it->second].trigger_event = (unsigned long long)ev;
                  e.num_triggers++;
                }
            events.push_back(e);
          }
    if ((int)cur_map.size() != c.grid[0] * c.grid[1] * c.grid[2])
      return fail(MK_EINVAL, "task graph: the partitions of '%s' and '%s' over their shared tensor leave blocks of '%s' without an event", p.name.c_str(),
                  c.name.c_str(), c.name.c_str());
    pre_map = cur_map;
  }
  // the last operator's tasks trigger END_OF_TASK_GRAPH
  const int end_ev = (int)events.size();
  for (auto &kv : pre_map)
    if (tasks[kv.second].trigger_event == REF_EVENT_INVALID) tasks[kv.second].trigger_event = (unsigned long long)end_ev;
  events.push_back({910 /*EVENT_END_OF_TASK_GRAPH*/, (int)pre_map.size(), 0, 0});
  events[1].last_task = (int)tasks.size();
  g->num_ref_tasks = (int)tasks.size();
  g->num_ref_events = (int)events.size();
  // sanity check (reference: runtime.cc:614-674): run the graph once from the first tasks; every task must run exactly
  // once, every event between operators fire exactly once, and END_OF_TASK_GRAPH be reached
  {
    std::vector<int> left(events.size()), fired(events.size(), 0), ran(tasks.size(), 0);
    for (size_t e = 0; e < events.size(); e++) left[e] = events[e].num_triggers;
    std::vector<int> queue(first_tasks.begin(), first_tasks.end());
    size_t head = 0;
    while (head < queue.size()) {
      const int k = queue[head++];
      if (ran[k]++) return fail(MK_EINVAL, "task graph sanity check: task %d scheduled twice", k);
      const unsigned long long ev = tasks[k].trigger_event;
      if (ev == REF_EVENT_INVALID) continue;
      if (left[ev] <= 0) return fail(MK_EINVAL, "task graph sanity check: event %llu triggered more often than it counts", ev);
      if (--left[ev] == 0) {
        if (fired[ev]++) return fail(MK_EINVAL, "task graph sanity check: event %llu fired twice", ev);
        if (events[ev].type == 900)
          for (int c2 = events[ev].first_task; c2 < events[ev].last_task; c2++) queue.push_back(c2);
      }
    }
    for (int k = 2; k < (int)tasks.size(); k++)
      if (ran[k] != 1) return fail(MK_EINVAL, "task graph sanity check: task %d ran %d times", k, ran[k]);
    for (int e = 2; e < end_ev; e++)
      if (fired[e] != 1) return fail(MK_EINVAL, "task graph sanity check: event %d fired %d times", e, fired[e]);
    if (!g->tasks.empty() && fired[end_ev] != 1) return fail(MK_EINVAL, "task graph sanity check: END_OF_TASK_GRAPH fired %d times", fired[end_ev]);
  }
  // variant ids: the reference registers one code variant per distinct instantiation of a task type (task_register.cc:
  // same constants -> same variant); restated here as: tasks of one type with the same name, per-block operand shapes and
  // params share a variant, numbered in order of first appearance
  std::vector<int> variant(g->tasks.size(), 0);
  {
    std::map<int, std::vector<std::string>> seen;  // task type -> signatures
    for (size_t oi = 0; oi < g->tasks.size(); oi++) {
      const Task &t = g->tasks[oi];
      std::string sig = t.name;
      for (size_t a = 0; a < t.ops.size(); a++) {
        sig += "|";
        if (t.ops[a] < 0) continue;
        const Tensor &tn = g->tensors[t.ops[a]];
        int part[4];
        partition_of(t, (int)a, part);
        for (int d = 0; d < tn.ndims; d++) sig += fmt("%lld,", (long long)(tn.dims[d] / std::gcd((long long)tn.dims[d], (long long)part[d])));
      }
      for (int v : t.params) sig += fmt(";%d", v);
      auto &lst = seen[task_type_id(t.name)];
      size_t k = 0;
      while (k < lst.size() && lst[k] != sig) k++;
      if (k == lst.size()) lst.push_back(sig);
      variant[oi] = (int)k;
    }
  }
  // JSON
  std::string &j = g->json;
  j.clear();
  j += "{\n \"all_tasks\": [\n";
  // one operand of one block: the slice the block's grid indices select (runtime.cc:1215-1414).  A shuffled (fused) tensor
  // is resolved to the source tensor and row the slice starts in (:1229-1283).
  auto operand_json = [&](const Task &t, size_t a, const int bid[3]) -> std::string {
    if (t.ops[a] < 0) return "{\"base_ptr\": \"nullptr\", \"offset\": 0, \"data_type\": 999, \"dims\": [], \"strides\": []}";
    const Tensor &tn = g->tensors[t.ops[a]];
    int part[4];
    partition_of(t, (int)a, part);
    long long dims[4];
    for (int d = 0; d < tn.ndims; d++) dims[d] = tn.dims[d] / std::gcd((long long)tn.dims[d], (long long)part[d]);
    const Tensor *base = &tn;
    long long off = 0;
    if (tn.kind == T_SHUFFLED) {
      const int groups = tn.interleave ? tn.num_groups : 1;
      std::vector<long long> gs;
      long long group_rows = 0;
      for (int sid : tn.sources) {
        gs.push_back(g->tensors[sid].dims[0] / groups);
        group_rows += gs.back();
      }
      long long row = 0;
      for (int ax = 0; ax < 3; ax++)
        if (t.maps[a][ax] == 0) row = tn.dims[0] / t.grid[ax] * bid[ax];
      long long in_group = row % group_rows;
      size_t si = 0;
      while (si + 1 < gs.size() && in_group >= gs[si]) in_group -= gs[si++];
      base = &g->tensors[tn.sources[si]];
      const long long sub_row = row / group_rows * gs[si] + in_group;
      for (int ax = 0; ax < 3; ax++) {
        const int d = t.maps[a][ax];
        if (d > 0 && d < base->ndims) off += base->dims[d] / t.grid[ax] * bid[ax] * base->strides[d];
        else if (d == 0) off += sub_row * base->strides[0];
      }
    } else {
      for (int ax = 0; ax < 3; ax++) {
        const int d = t.maps[a][ax];
        if (d >= 0 && d < tn.ndims) off += tn.dims[d] / t.grid[ax] * bid[ax] * tn.strides[d];
      }
    }
    std::string e = fmt("{\"base_ptr\": \"%s\", \"offset\": %lld, \"data_type\": %d, \"dims\": [", base->name.c_str(), off * (long long)dtype_size(base->dtype), tn.dtype);
    for (int d = 0; d < tn.ndims; d++) e += fmt(d ? ", %lld" : "%lld", dims[d]);
    e += "], \"strides\": [";
    for (int d = 0; d < tn.ndims; d++) e += fmt(d ? ", %lld" : "%lld", (long long)base->strides[d]);
    e += "]}";
    return e;
  };
  for (size_t k = 0; k < tasks.size(); k++) {
    const RefTask &rt = tasks[k];
    const int type = k == 0 ? 0 /*TASK_TERMINATE*/ : (k == 1 ? 10 /*TASK_BEGIN_TASK_GRAPH*/ : task_type_id(g->tasks[rt.op_index].name));
    j += fmt("  {\"task_type\": %d, \"variant_id\": %d, \"inputs\": [", type, rt.op_index >= 0 ? variant[rt.op_index] : 0);
    std::string outs;
    unsigned long long meta = ~0ull;
    if (rt.op_index >= 0) {
      const Task &t = g->tasks[rt.op_index];
      const int n_in = (int)t.ops.size() - num_outputs(t);
      for (size_t a = 0; a < t.ops.size(); a++) {
        const std::string e = operand_json(t, a, rt.bid);
        if ((int)a < n_in) j += ((int)a ? ", " : "") + e;
        else outs += ((int)a > n_in ? ", " : "") + e;
      }
      meta = ref_task_metadata(t, rt.bid);
    }
    j += "], \"outputs\": [" + outs + "], ";
    j += fmt("\"trigger_event\": %llu, \"dependent_event\": %llu, \"request_id\": %d, \"expert_offset\": %d, \"kv_idx\": %d, "
             "\"merge_task_offset\": %d, \"n_tile_start\": %d, \"n_tile_count\": %d}%s\n",
             rt.trigger_event, rt.dependent_event, k < 2 ? -1 : (int)(int16_t)(meta & 0xffff), k < 2 ? -1 : (int)(int32_t)(meta & 0xffffffffu),
             k < 2 ? -1 : (int)((meta >> 16) & 0xffff), k < 2 ? -1 : (int)(int32_t)(meta >> 32), k < 2 ? 0 : (int)(meta & 0xffff),
             k < 2 ? 0 : (int)((meta >> 16) & 0xffff), k + 1 < tasks.size() ? "," : "");
  }
  j += " ],\n \"all_events\": [\n";
  for (size_t e = 0; e < events.size(); e++)
    j += fmt("  {\"event_type\": %d, \"num_triggers\": %d, \"first_task_id\": %d, \"last_task_id\": %d}%s\n", events[e].type, events[e].num_triggers,
             events[e].first_task, events[e].last_task, e + 1 < events.size() ? "," : "");
  j += " ],\n \"first_tasks\": [";
  for (size_t k = 0; k < first_tasks.size(); k++) j += fmt(k ? ", %d" : "%d", first_tasks[k]);
  j += "]\n}\n";
  return MK_OK;
}

int upload_runtime(mk_graph *g) {
  HIP_TRY(hipMemcpy(g->d_rt, &g->h_rt, sizeof(MkRuntime), hipMemcpyHostToDevice));
  return MK_OK;
}

// `rt` is the runtime block the kernel receives by value; `cleared_by_caller`: its barrier state has been zeroed already
// graphs with flex stages (mk_flex.hip) have kernels of their own; graphs that never run more than one token per iteration
// use the instantiation for exactly that.  Null: not in this build of the library.
static const void *kernel_of(const mk_graph *g) {
  const bool m1 = g->cfg.max_num_batched_tokens == 1;
  const void *k = nullptr;
  if (g->flex == FLEX_NONE) {
#ifdef MK_HAVE_KERNEL_DENSE
    k = m1 ? (const void *)mk_persistent_kernel_m1 : (const void *)mk_persistent_kernel;
#endif
  } else if (g->dual) {
#ifdef MK_HAVE_KERNEL_DUAL
    if (g->flex == FLEX_BF16 && !m1) k = (const void *)mk_persistent_kernel_dual;
#endif
#ifdef MK_HAVE_KERNEL_DUAL_M1
    if (g->flex == FLEX_BF16 && m1) k = (const void *)mk_persistent_kernel_dual_m1;
#endif
#ifdef MK_HAVE_KERNEL_DUAL_F32
    if (g->flex == FLEX_F32) k = (const void *)mk_persistent_kernel_dual_f32;
#endif
  } else if (g->hyb) {
#ifdef MK_HAVE_KERNEL_HYB
    if (g->flex == FLEX_BF16 && !m1) k = (const void *)mk_persistent_kernel_hyb;
#endif
#ifdef MK_HAVE_KERNEL_HYB_M1
    if (g->flex == FLEX_BF16 && m1) k = (const void *)mk_persistent_kernel_hyb_m1;
#endif
#ifdef MK_HAVE_KERNEL_HYB_F32
    if (g->flex == FLEX_F32) k = (const void *)mk_persistent_kernel_hyb_f32;
#endif
  } else if (g->mix) {
#ifdef MK_HAVE_KERNEL_MIX
    if (g->flex == FLEX_BF16 && !m1) k = (const void *)mk_persistent_kernel_mix;
#endif
#ifdef MK_HAVE_KERNEL_MIX_M1
    if (g->flex == FLEX_BF16 && m1) k = (const void *)mk_persistent_kernel_mix_m1;
#endif
#ifdef MK_HAVE_KERNEL_MIX_F32
    if (g->flex == FLEX_F32) k = (const void *)mk_persistent_kernel_mix_f32;
#endif
  } else if (g->flex == FLEX_BF16) {
#ifdef MK_HAVE_KERNEL_FLEX
    if (!m1) k = (const void *)mk_persistent_kernel_flex;
#endif
#ifdef MK_HAVE_KERNEL_FLEX_M1
    if (m1) k = (const void *)mk_persistent_kernel_flex_m1;
#endif
  } else {
#ifdef MK_HAVE_KERNEL_FLEX_F32
    k = (const void *)mk_persistent_kernel_flex_f32;
#endif
  }
  (void)m1;
  return k;
}

int do_launch(mk_graph *g, hipStream_t stream, int max_iters, int run_scheduler, const MkRuntime *rt = nullptr, bool cleared_by_caller = false) {
  if (!g->compiled) return fail(MK_ESTATE, "mk_compile has not been called");
  if (g->launch_pending) return fail(MK_ESTATE, "a launch is still pending: call mk_wait first");
  HIP_TRY(hipSetDevice(g->cfg.device));
  if (!rt) rt = &g->h_rt;
  if (!cleared_by_caller) HIP_TRY(hipMemsetAsync(rt->sync, 0, sizeof(MkSync), stream));
  const MkRuntime *rtp = g->d_rt;
  void *args[] = {(void *)rt, (void *)&rtp, (void *)&max_iters, (void *)&run_scheduler};
  HIP_TRY(hipEventRecord(g->ev0, stream));
  HIP_TRY(hipLaunchCooperativeKernel(kernel_of(g), dim3(g->G), dim3(MK_THREADS), args, MK_LDS_BYTES, stream));
  HIP_TRY(hipEventRecord(g->ev1, stream));
  g->launch_pending = true;
  g->pending_sync = rt->sync;
  return MK_OK;
}

int do_wait(mk_graph *g, hipStream_t stream, int *finished_out) {
  if (!g->launch_pending) return fail(MK_ESTATE, "no launch pending");
  HIP_TRY(hipStreamSynchronize(stream));
  g->launch_pending = false;
  float ms = 0.f;
  HIP_TRY(hipEventElapsedTime(&ms, g->ev0, g->ev1));
  g->last_ms = ms;
  MkSync hs;
  HIP_TRY(hipMemcpy(&hs, g->pending_sync ? g->pending_sync : g->d_sync, sizeof(MkSync), hipMemcpyDeviceToHost));
  int nx = 0;
  for (int i = 0; i < MK_MAX_XCD; i++) nx += hs.xcd_count[i] > 0;
  g->last_nxcd = nx;
  g->last_aborted = hs.abort_flag != 0;
  MkSched sc;
  HIP_TRY(hipMemcpy(&sc, g->d_sched, sizeof(MkSched), hipMemcpyDeviceToHost));
  if (finished_out) *finished_out = sc.finished;
  if (hs.abort_flag) {
    // workgroups that unwound mid-stage may have left the split-K and split-KV arrival counters mid-count (their last
    // arriver resets them); the next launch on this handle must not inherit that
    HIP_TRY(hipMemset(g->h_rt.attn_cnt, 0, sizeof(unsigned) * g->attn_cnt_n));
    HIP_TRY(hipMemset(g->h_rt.splitk_cnt, 0, sizeof(unsigned) * 32 * (size_t)g->G));
    return fail(MK_EABORT, "kernel watchdog fired (barrier epoch %u): a workgroup waited longer than the spin limit", hs.abort_where);
  }
  if (sc.bad_batch) {
    static const char *why[] = {"", "rows outside [0, max_num_batched_tokens), overlapping, or with gaps", "more rows for one request than max_tokens_per_request",
                                "a sequence shorter than its new rows, longer than max_seq_length, or without pages"};
    return fail(MK_EINVAL, "the batch described in qo_indptr / paged_kv_* was rejected and nothing was run: %s", why[sc.bad_batch > 0 && sc.bad_batch <= 3 ? sc.bad_batch : 1]);
  }
  return MK_OK;
}

// ---- launch scratch that no call allocates -------------------------------------------------------------------
// mk_enqueue_steps_static runs a compiled graph with every piece of launch scratch -- the grid barrier's counters, the
// K-split partial tiles and their arrival counters, the attention stages' split-KV partials and counters, the
// sampling stages' per-workgroup partials -- taken from this file-scope device array instead of from the buffers
// mk_compile allocated.  Each GPU the library runs on holds its own copy of the array until the process ends.
// Sizes are for the largest launch the entry point accepts (256 workgroups, 64 tokens x 8 kv heads, 8 q heads per kv head).
constexpr size_t align256(size_t n) { return (n + 255) / 256 * 256; }
constexpr int MK_STATIC_MAX_WG = 256;
constexpr int MK_STATIC_MAX_ITEMS = MK_MAX_TOKENS * 8;  // (token, kv head) pairs
constexpr int MK_STATIC_MAX_QPK = 8;
constexpr size_t SS_SYNC = 0;
constexpr size_t SS_SPLITK_CNT = SS_SYNC + align256(sizeof(MkSync));
constexpr size_t SS_ATTN_CNT = SS_SPLITK_CNT + align256((size_t)MK_STATIC_MAX_WG * 32 * sizeof(unsigned));
constexpr size_t SS_CLEARED_END = SS_ATTN_CNT + align256((size_t)MK_STATIC_MAX_ITEMS * 32 * sizeof(unsigned));  // [0, here) starts every call at zero
constexpr size_t SS_ARGMAX_PV = SS_CLEARED_END;
constexpr size_t SS_ARGMAX_PI = SS_ARGMAX_PV + align256((size_t)MK_MAX_TOKENS * MK_STATIC_MAX_WG * sizeof(float));
constexpr size_t SS_ATTN_PART = SS_ARGMAX_PI + align256((size_t)MK_MAX_TOKENS * MK_STATIC_MAX_WG * sizeof(int));
// q-head partials of the attention stages: at most max(workgroups, (token, kv head) pairs) work units of up to 8 q heads each
constexpr size_t MK_STATIC_ATTN_HEADS = (size_t)std::max(MK_STATIC_MAX_ITEMS, MK_STATIC_MAX_WG) * MK_STATIC_MAX_QPK;
constexpr size_t SS_SPLITK_PART = SS_ATTN_PART + align256(MK_STATIC_ATTN_HEADS * MK_ATTN_PSTRIDE * sizeof(float));
constexpr size_t MK_STATIC_SCRATCH_BYTES = SS_SPLITK_PART + (size_t)MK_STATIC_MAX_WG * 4 * 4 * 4 * 64 * 16;  // about 19.6 MB

static __device__ __align__(256) unsigned char scratch[MK_STATIC_SCRATCH_BYTES];

constexpr int MK_MAX_DEVICES = 64;
unsigned char *g_scratch_ptr[MK_MAX_DEVICES];  // device address of `scratch` on each device, resolved once per device

// `scratch` is a host-side stand-in in host code, not a device address: the address every kernel argument, fill and
// copy uses is the one hipGetSymbolAddress returns, asked for once per device with that device current.
int resolve_scratch(int device) {
  if (device < 0 || device >= MK_MAX_DEVICES) return fail(MK_EINVAL, "device %d outside [0, %d)", device, MK_MAX_DEVICES);
  if (g_scratch_ptr[device]) return MK_OK;
  HIP_TRY(hipSetDevice(device));
  void *p = nullptr;
  HIP_TRY(hipGetSymbolAddress(&p, HIP_SYMBOL(scratch)));
  if (!p) return fail(MK_EHIP, "hipGetSymbolAddress returned a null address for the launch scratch");
  g_scratch_ptr[device] = (unsigned char *)p;
  return MK_OK;
}

// zero-fill by kernel (a fill node that a caller's graph capture records safely, unlike a memset node)
__global__ void mk_fill_zero_kernel(uint4 *p, size_t n16) {
  const uint4 z = {0u, 0u, 0u, 0u};
  for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n16; i += (size_t)gridDim.x * blockDim.x) p[i] = z;
}

}  // namespace

// ============================================================================ C ABI
extern "C" {

const char *mk_last_error(void) { return g_err.c_str(); }
const char *mk_version(void) { return "fleet_mk 0.1 (gfx950)"; }

int mk_graph_create(const mk_config *cfg, mk_graph **out) {
  if (!cfg || !out) return fail(MK_EINVAL, "null argument");
  if (cfg->max_num_batched_tokens < 1 || cfg->max_num_batched_tokens > MK_MAX_TOKENS)
    return fail(MK_EINVAL, "max_num_batched_tokens=%d outside [1, %d]", cfg->max_num_batched_tokens, MK_MAX_TOKENS);
  if (cfg->max_num_batched_requests < 1 || cfg->max_num_batched_requests > MK_MAX_TOKENS)
    return fail(MK_EINVAL, "max_num_batched_requests=%d outside [1, %d]", cfg->max_num_batched_requests, MK_MAX_TOKENS);
  if (cfg->mode < MK_MODE_OFFLINE || cfg->mode > MK_MODE_ONEPASS) return fail(MK_EINVAL, "mode=%d is not one of enum mk_mode", cfg->mode);
  if (cfg->max_tokens_per_request < 0 || cfg->max_tokens_per_request > MK_MAX_NEW_PER_REQ)
    return fail(MK_EINVAL, "max_tokens_per_request=%d outside [0, %d]", cfg->max_tokens_per_request, MK_MAX_NEW_PER_REQ);
  if (cfg->page_size < 1 || cfg->max_num_pages < 1 || cfg->max_seq_length < 2) return fail(MK_EINVAL, "bad page_size / max_num_pages / max_seq_length");
  if ((int64_t)cfg->max_num_pages * cfg->page_size < cfg->max_seq_length)
    return fail(MK_EINVAL, "max_num_pages*page_size=%lld cannot hold one sequence of max_seq_length=%d", (long long)cfg->max_num_pages * cfg->page_size,
                cfg->max_seq_length);
  // The next two limits protect state only the on-GPU schedulers keep (MK_MODE_OFFLINE, MK_MODE_ONLINE): their page ring
  // and the LDS snapshot of the page table.  In MK_MODE_ONLINE_NOTOKEN / MK_MODE_ONEPASS the host owns the page table;
  // max_num_pages is then the serving engine's block count, which may be oversubscribed and much larger.
  const bool gpu_pages = cfg->mode == MK_MODE_OFFLINE || cfg->mode == MK_MODE_ONLINE;
  if (gpu_pages) {
    // Every slot can grow to max_seq_length, and the page ring (like the reference's) hands out pages without checking
    // that any are free: with fewer pages than that a page would be given to two requests.
    const int64_t per_req = ((int64_t)cfg->max_seq_length + cfg->page_size - 1) / cfg->page_size;
    if (per_req * cfg->max_num_batched_requests > cfg->max_num_pages)
      return fail(MK_EINVAL, "max_num_pages=%d cannot back %d concurrent requests of up to %lld pages each (max_seq_length=%d, page_size=%d)",
                  cfg->max_num_pages, cfg->max_num_batched_requests, (long long)per_req, cfg->max_seq_length, cfg->page_size);
    if (cfg->max_num_pages > (MK_LDS_BYTES / 8)) return fail(MK_EINVAL, "max_num_pages=%d exceeds the scheduler's LDS snapshot (%d)", cfg->max_num_pages, MK_LDS_BYTES / 8);
  }
  if (((int64_t)cfg->max_seq_length + cfg->page_size - 1) / cfg->page_size > MK_ATTN_MAX_REQ_PAGES)
    return fail(MK_EINVAL, "max_seq_length=%d over page_size=%d is more than %d pages per request (the attention stage keeps a request's page list in LDS)",
                cfg->max_seq_length, cfg->page_size, MK_ATTN_MAX_REQ_PAGES);
  if (cfg->device < 0) {
    mk_graph *g = new mk_graph();
    g->cfg = *cfg;
    if (g->cfg.rms_eps == 0.f) g->cfg.rms_eps = 1e-6f;
    g->host_only = true;
    g->num_cus = 256;
    g->G = cfg->num_workers > 0 ? cfg->num_workers : 256;
    memset(&g->h_rt, 0, sizeof(g->h_rt));
    *out = g;
    return MK_OK;
  }
  int ndev = 0;
  HIP_TRY(hipGetDeviceCount(&ndev));
  if (ndev < 1) return fail(MK_EHIP, "no HIP device visible: the megakernel has no CPU fallback");
  if (cfg->device < 0 || cfg->device >= ndev) return fail(MK_EINVAL, "device %d out of range", cfg->device);
  HIP_TRY(hipSetDevice(cfg->device));
  hipDeviceProp_t prop;
  HIP_TRY(hipGetDeviceProperties(&prop, cfg->device));
  if (strncmp(prop.gcnArchName, "gfx950", 6) != 0) return fail(MK_EUNSUPPORTED, "device is %s; this library is built for gfx950 only", prop.gcnArchName);
  if (!prop.cooperativeLaunch) return fail(MK_EUNSUPPORTED, "device does not support cooperative launch");
  mk_graph *g = new mk_graph();
  g->cfg = *cfg;
  if (g->cfg.rms_eps == 0.f) g->cfg.rms_eps = 1e-6f;
  g->num_cus = prop.multiProcessorCount;
  g->G = cfg->num_workers > 0 ? cfg->num_workers : g->num_cus;
  if (g->G > g->num_cus) {
    delete g;
    return fail(MK_EINVAL, "num_workers=%d exceeds the %d CUs that can be co-resident", cfg->num_workers, prop.multiProcessorCount);
  }
  memset(&g->h_rt, 0, sizeof(g->h_rt));
  *out = g;
  return MK_OK;
}

int mk_graph_destroy(mk_graph *g) {
  if (!g) return MK_OK;
  if (g->launch_pending) (void)hipDeviceSynchronize();
  for (void *p : g->allocs) (void)hipFree(p);
  for (void *p : g->host_allocs) free(p);
  if (g->ev0) (void)hipEventDestroy(g->ev0);
  if (g->ev1) (void)hipEventDestroy(g->ev1);
  delete g;
  return MK_OK;
}

static int add_tensor(mk_graph *g, Tensor &&t) {
  g->tensors.push_back(std::move(t));
  return (int)g->tensors.size() - 1;
}

int mk_tensor_attach(mk_graph *g, void *device_ptr, int ndims, const int64_t *dims, const int64_t *strides, int dtype, const char *name) {
  if (!g || !dims || !name) return fail(MK_EINVAL, "null argument");
  if (g->compiled) return fail(MK_ESTATE, "graph already compiled");
  if (ndims < 1 || ndims > 4) return fail(MK_EINVAL, "tensor '%s': %d dims (1..4 supported)", name, ndims);
  if (!dtype_size(dtype)) return fail(MK_EINVAL, "tensor '%s': unsupported dtype %d", name, dtype);
  if (!device_ptr) return fail(MK_EINVAL, "tensor '%s': null device pointer", name);
  Tensor t;
  t.name = name;
  t.ndims = ndims;
  t.dtype = dtype;
  t.kind = T_ATTACHED;
  t.ptr = device_ptr;
  int64_t expect = 1;
  for (int i = ndims - 1; i >= 0; i--) {
    t.dims[i] = dims[i];
    t.strides[i] = strides ? strides[i] : expect;
    if (t.strides[i] != expect) return fail(MK_EINVAL, "tensor '%s' is not row-major contiguous (stride[%d]=%lld, expected %lld)", name, i, (long long)t.strides[i], (long long)expect);
    expect *= dims[i];
  }
  return add_tensor(g, std::move(t));
}

int mk_tensor_new(mk_graph *g, int ndims, const int64_t *dims, const int64_t *strides, int dtype, const char *name, int io_category) {
  if (!g || !dims || !name) return fail(MK_EINVAL, "null argument");
  if (g->compiled) return fail(MK_ESTATE, "graph already compiled");
  if (ndims < 1 || ndims > 4) return fail(MK_EINVAL, "tensor '%s': %d dims (1..4 supported)", name, ndims);
  if (!dtype_size(dtype)) return fail(MK_EINVAL, "tensor '%s': unsupported dtype %d", name, dtype);
  if (io_category != MK_IO_DEVICE && io_category != MK_IO_SYMMETRIC) return fail(MK_EINVAL, "Invalid io_category: %d", io_category);
  Tensor t;
  t.name = name;
  t.ndims = ndims;
  t.dtype = dtype;
  t.kind = T_OWNED;
  t.io_category = io_category;
  int64_t expect = 1;
  size_t span = 1;
  for (int i = ndims - 1; i >= 0; i--) {
    t.dims[i] = dims[i];
    t.strides[i] = strides ? strides[i] : expect;
    expect *= dims[i];
    span += (size_t)(dims[i] - 1) * (size_t)t.strides[i];
  }
  // allocate right away so later tasks can capture the address; freed in mk_graph_destroy
  void *p = nullptr;
  int rc = dev_alloc(g, &p, span * dtype_size(dtype));
  if (rc) return rc;
  t.ptr = p;
  return add_tensor(g, std::move(t));
}

int mk_tensor_shuffle(mk_graph *g, const int *ids, int n, int dim, int num_groups, int interleave, const char *name) {
  if (!g || !ids || !name) return fail(MK_EINVAL, "null argument");
  if (dim != 0) return fail(MK_EUNSUPPORTED, "only dimension 0 can be shuffled/fused");
  if (n < 1 || n > MK_MAX_SEGS) return fail(MK_EUNSUPPORTED, "shuffle of %d tensors (1..%d supported)", n, MK_MAX_SEGS);
  if (num_groups < 1) return fail(MK_EINVAL, "num_groups must be positive");
  Tensor t;
  t.name = name;
  t.kind = T_SHUFFLED;
  t.num_groups = num_groups;
  t.interleave = interleave != 0;
  int64_t rows = 0;
  for (int i = 0; i < n; i++) {
    if (ids[i] < 0 || ids[i] >= (int)g->tensors.size()) return fail(MK_EINVAL, "bad tensor id %d", ids[i]);
    const Tensor &s = g->tensors[ids[i]];
    if (s.ndims != 2) return fail(MK_EINVAL, "shuffle source '%s' must be 2-D", s.name.c_str());
    if (i && (s.dims[1] != g->tensors[ids[0]].dims[1] || s.dtype != g->tensors[ids[0]].dtype)) return fail(MK_EINVAL, "shuffle sources disagree on columns/dtype");
    if (s.dims[0] % num_groups) return fail(MK_EINVAL, "source '%s' rows %lld not divisible by num_groups %d", s.name.c_str(), (long long)s.dims[0], num_groups);
    rows += s.dims[0];
    t.sources.push_back(ids[i]);
  }
  t.ndims = 2;
  t.dtype = g->tensors[ids[0]].dtype;
  t.dims[0] = rows;
  t.dims[1] = g->tensors[ids[0]].dims[1];
  t.strides[0] = t.dims[1];
  t.strides[1] = 1;
  return add_tensor(g, std::move(t));
}

int mk_tensor_num_dims(mk_graph *g, int id) {
  if (!g || id < 0 || id >= (int)g->tensors.size()) return fail(MK_EINVAL, "bad tensor id %d", id);
  return g->tensors[id].ndims;
}
int64_t mk_tensor_dim(mk_graph *g, int id, int i) {
  if (!g || id < 0 || id >= (int)g->tensors.size()) return fail(MK_EINVAL, "bad tensor id %d", id);
  if (i < 0 || i >= g->tensors[id].ndims) return fail(MK_EINVAL, "bad dim %d", i);
  return g->tensors[id].dims[i];
}
void *mk_tensor_ptr(mk_graph *g, int id) {
  if (!g || id < 0 || id >= (int)g->tensors.size()) return nullptr;
  return g->tensors[id].ptr;
}

int mk_add_task(mk_graph *g, const char *task_name, const int grid_dim[3], const int block_dim[3], int n_operands, const int *tensor_ids,
                const int *input_maps, const int *forloop_dims, int n_params, const int *params) {
  if (!g || !task_name || !grid_dim || !block_dim || (n_operands > 0 && !tensor_ids)) return fail(MK_EINVAL, "null argument");
  if (g->compiled) return fail(MK_ESTATE, "graph already compiled");
  Task t;
  t.name = task_name;
  for (int i = 0; i < 3; i++) {
    t.grid[i] = grid_dim[i];
    t.block[i] = block_dim[i];
    if (grid_dim[i] < 1) return fail(MK_EINVAL, "task '%s': grid_dim[%d]=%d", task_name, i, grid_dim[i]);
  }
  for (int i = 0; i < n_operands; i++) {
    // id -1 = optional operand that is absent: only the q/k-norm weights and the cos/sin tables of the attention tasks
    // (and the sink of flex_attention, the summand of residual_rmsnorm, what the mix tasks may leave out)
    const bool optional = ((t.name == "gang_attn_split_kv_mi300" || t.name == "kv_cache_update_mi300" || t.name == "paged_attention" ||
                           t.name == "paged_attention_split_kv_mi300" || t.name == "attention" || t.name == "single_batch_extend_attention") && i >= 3 && i <= 6) ||
                          (t.name == "flex_attention" && i >= 3 && i <= (n_operands == 12 ? 9 : n_operands == 9 ? 6 : 5)) || (t.name == "expert_linear" && i == 2) || (t.name == "residual_rmsnorm" && i == 0) ||
                          (t.name == "residual_prenorm" && (i == 0 || i == 1 || i == 3 || (n_operands == 8 && (i == 2 || i == 5)) || (n_operands == 11 && i != 7 && i != 10))) || (t.name == "latent_prep" && i >= 1 && i <= 7) ||
                          (t.name == "head_linear" && (i == 2 || i == 3)) || (t.name == "latent_attention" && (i == 3 || i == 4)) || (t.name == "general_delta" && i == 8) ||
                          (t.name == "ring_conv" && (i == 2 || i == 5 || i == 6 || i == 8));
    if (tensor_ids[i] >= (int)g->tensors.size() || tensor_ids[i] < (optional ? -1 : 0))
      return fail(MK_EINVAL, "task '%s': bad tensor id %d for operand %d", task_name, tensor_ids[i], i);
    t.ops.push_back(tensor_ids[i]);
    std::array<int, 3> m = {-1, -1, -1};
    if (input_maps) m = {input_maps[3 * i], input_maps[3 * i + 1], input_maps[3 * i + 2]};
    t.maps.push_back(m);
    t.forloop.push_back(forloop_dims ? forloop_dims[i] : -1);
  }
  for (int i = 0; i < n_params; i++) t.params.push_back(params[i]);
  // reject unknown names here, like Graph::register_task (src/kernel/graph.cc:844-847)
  bool a, b;
  int c;
  static const char *known[] = {"embedding", "rmsnorm", "gang_rmsnorm_mi300", "silu_mul", "gang_attn_split_kv_mi300", "kv_cache_update_mi300",
                                "paged_attention_ck_fmha_split_kv_mi300", "argmax_partial", "argmax_reduce", "moe_topk_softmax_mi300", "moe_w13_linear_mi300",
                                "moe_w2_linear_mi300", "gang_moe_w13_linear_mi300", "gang_moe_w2_linear_mi300", "moe_silu_mul", "moe_mul_sum_add_mi300",
                                "paged_attention", "paged_attention_split_kv_mi300", "paged_attention_split_kv_merge_mi300",
                                "paged_attention_ck_fmha_merge_mi300", "gang_attn_merge_mi300", "splitk_reduce_mi300", "silu_mul_linear_with_residual", "rmsnorm_linear", "identity", "argmax", "attention",
                                "find_ngram_partial", "find_ngram_global", "target_verify_greedy", "single_batch_extend_attention",
                                "embedding_scaled", "residual_rmsnorm", "flex_attention", "residual_prenorm", "latent_prep", "head_linear", "latent_attention", "general_delta",
                                "relu_squared", "short_conv", "scan_step", "selective_scan", "expert_route", "expert_linear", "ring_conv", "dual_scan", "gelu_mul"};
  bool ok = linear_kind(t.name, &a, &b, &c);
  for (auto k : known) ok = ok || t.name == k;
  if (!ok) return fail(MK_EUNSUPPORTED, "Unsupported task name: %s", task_name);
  g->tasks.push_back(std::move(t));
  return MK_OK;
}

int mk_generate_task_graph(mk_graph *g, int num_gpus, int my_gpu_id, const char **json_out) {
  if (!g || !json_out) return fail(MK_EINVAL, "null argument");
  if (num_gpus != 1 || my_gpu_id != 0) return fail(MK_EUNSUPPORTED, "this build runs on one GPU (num_gpus=%d, my_gpu_id=%d)", num_gpus, my_gpu_id);
  int rc = build_task_graph_json(g);
  if (rc) return rc;
  *json_out = g->json.c_str();
  return MK_OK;
}

// Matrix-core copies of the linear weights (MkStage::wpack).  A graph that can run more than eight tokens per iteration
// streams its weights through the matrix cores in 16-row tiles; read from a row-major matrix that is 64 bytes from each
// of 16 rows per request, which HBM serves at about three quarters of the rate of one contiguous stream.  So every such
// weight is re-laid once, tile by tile, in a buffer the handle owns (this doubles the weight footprint; single-token
// iterations keep reading the caller's row-major tensors).  FLEET_MK_PACK_WEIGHTS=0 turns the copies off.
// allocate = false re-runs the copy kernels into the existing buffers (the caller changed weights after compiling).
static int pack_weights(mk_graph *g, bool allocate) {
  const char *env = getenv("FLEET_MK_PACK_WEIGHTS");
  if (g->cfg.max_num_batched_tokens < 2 || (env && atoi(env) == 0)) return 0;
  for (auto &st : g->stages) {
    if (st.op != MK_OP_LINEAR || (st.k & 63) || st.k < 64) continue;
    const bool silu = st.flags & MK_F_SILU;
    const int n_out = silu ? st.n / 2 : st.n;
    const long long tiles = (long long)((n_out + 15) / 16) * (silu ? 2 : 1);
    const long long total = tiles * (st.k >> 6) * 128;  // 16-byte operands
    if (allocate) {
      void *p = nullptr;
      if (hipMalloc(&p, (size_t)total * 16) != hipSuccess) {
        (void)hipGetLastError();
        return fail(MK_EHIP, "no device memory for the %.1f MB matrix-core copy of a weight (FLEET_MK_PACK_WEIGHTS=0 runs without the copies)", total * 16 / 1e6);
      }
      g->allocs.push_back(p);
      st.wpack = p;
      g->packed_bytes += total * 16;
    }
    if (!st.wpack) continue;
    hipLaunchKernelGGL(mk_pack_weights_kernel, dim3(2048), dim3(256), 0, 0, st.w, st.n, st.k, silu ? 1 : 0, st.silu_half, (u32x4 *)st.wpack, total);
    HIP_TRY(hipGetLastError());
  }
  HIP_TRY(hipDeviceSynchronize());
  return 0;
}

int mk_repack_weights(mk_graph *g) {
  if (!g) return fail(MK_EINVAL, "null argument");
  if (!g->compiled) return fail(MK_ESTATE, "graph not compiled");
  if (g->single_copy) return fail(MK_ESTATE, "this graph keeps only the tile copies of its weights (MK_CFG_SINGLE_WEIGHT_COPY): the row-major tensors may be gone");
  HIP_TRY(hipSetDevice(g->cfg.device));
  return pack_weights(g, false);
}

int mk_tensor_releasable(mk_graph *g, int id) {
  if (!g || id < 0 || id >= (int)g->tensors.size()) return fail(MK_EINVAL, "bad tensor id %d", id);
  if (!g->compiled || id >= (int)g->releasable.size()) return 0;
  return g->releasable[id] ? 1 : 0;
}

int mk_compile(mk_graph *g) {
  if (!g) return fail(MK_EINVAL, "null argument");
  if (g->compiled) return fail(MK_ESTATE, "graph already compiled");
  if (g->host_only) return fail(MK_ESTATE, "this graph was created without a device (device < 0): it can be lowered and described, not compiled");
  HIP_TRY(hipSetDevice(g->cfg.device));
  const mk_config &c = g->cfg;
  if (!c.step || !c.tokens || !c.input_tokens || !c.output_tokens || !c.prompt_lengths || !c.qo_indptr || !c.paged_kv_indptr || !c.paged_kv_indices ||
      !c.paged_kv_last_page_len)
    return fail(MK_EINVAL, "all meta tensors except num_new_tokens must be non-null device pointers");
  int rc = lower(g);
  if (rc) return rc;
  rc = build_task_graph_json(g);
  if (rc) return rc;
  if (!kernel_of(g)) return fail(MK_EUNSUPPORTED, "this build of the library leaves out the kernel this graph runs on");
  // co-residency: every workgroup must be resident for the in-kernel barriers to make progress
  HIP_TRY(hipFuncSetAttribute(kernel_of(g), hipFuncAttributeMaxDynamicSharedMemorySize, MK_LDS_BYTES));
  int per_cu = 0;
  HIP_TRY(hipOccupancyMaxActiveBlocksPerMultiprocessor(&per_cu, kernel_of(g), MK_THREADS, MK_LDS_BYTES));
  if (per_cu < 1 || g->G > per_cu * g->num_cus) return fail(MK_EINVAL, "grid of %d workgroups cannot be co-resident (%d per CU x %d CUs)", g->G, per_cu, g->num_cus);
  MkRuntime &rt = g->h_rt;
  rt.num_stages = (int)g->stages.size();
  rt.max_tokens = c.max_num_batched_tokens;
  rt.max_requests = c.max_num_batched_requests;
  rt.max_seq = c.max_seq_length;
  rt.page_size = c.page_size;
  rt.max_pages = c.max_num_pages;
  rt.total_requests = c.total_num_requests;
  rt.max_new_per_req = c.max_tokens_per_request > 0 ? c.max_tokens_per_request : 8;
  rt.spec_len = g->spec_len;
  rt.state_ids = g->state_ids;
  rt.eos_token_id = c.eos_token_id;
  rt.step = c.step;
  rt.tokens = (long long *)c.tokens;
  rt.input_tokens = (long long *)c.input_tokens;
  rt.output_tokens = (long long *)c.output_tokens;
  rt.num_new_tokens = c.num_new_tokens;
  rt.prompt_lengths = c.prompt_lengths;
  rt.qo_indptr = c.qo_indptr;
  rt.kv_indptr = c.paged_kv_indptr;
  rt.kv_indices = c.paged_kv_indices;
  rt.kv_last_page_len = c.paged_kv_last_page_len;
  void *p;
  if ((rc = dev_alloc(g, &p, sizeof(int) * rt.max_requests))) return rc;
  rt.request_ids = (int *)p;
  if ((rc = dev_alloc(g, &p, sizeof(int) * rt.max_pages))) return rc;
  rt.page_queue = (int *)p;
  if ((rc = dev_alloc(g, &p, sizeof(int) * rt.max_tokens))) return rc;
  rt.tok_slot = (int *)p;
  if ((rc = dev_alloc(g, &p, sizeof(int) * rt.max_tokens))) return rc;
  rt.tok_pos = (int *)p;
  if ((rc = dev_alloc(g, &p, sizeof(int) * rt.max_tokens))) return rc;
  rt.tok_first = (int *)p;
  if ((rc = dev_alloc(g, &p, sizeof(MkSched)))) return rc;
  rt.sched = g->d_sched = (MkSched *)p;
  if ((rc = dev_alloc(g, &p, sizeof(MkSync)))) return rc;
  rt.sync = g->d_sync = (MkSync *)p;
  // attention split-KV workspace: one partial (max, sum, 128 values) per q head of every work unit, a buffer of its
  // own for every attention stage (a partial address is then written once per iteration), and two sets of arrival
  // counters (device scope / die-local), one 128-byte line per (token, kv head)
  int max_kv = 1;
  for (auto &s : g->stages)
    if (s.op == MK_OP_ATTN) {
      if (s.num_kv_heads > max_kv) max_kv = s.num_kv_heads;
      g->max_qpk = std::max(g->max_qpk, s.num_q_heads / s.num_kv_heads);
    }
  g->max_kv_heads = max_kv;
  g->attn_cnt_n = std::max((size_t)rt.max_tokens * max_kv * 2, g->flex_items) * 32;
  if ((rc = dev_alloc(g, &p, sizeof(unsigned) * g->attn_cnt_n))) return rc;
  rt.attn_cnt = (unsigned *)p;
  rt.attn_part = nullptr;
  if (g->flex_part) {
    // the flex attention stages share one buffer of chunk partials, handed over at device scope
    if ((rc = dev_alloc(g, &p, g->flex_part * sizeof(float), false))) return rc;
    rt.attn_part = (float *)p;
  }
  for (auto &s : g->stages)
    if (s.op == MK_OP_ATTN) {
      // a work unit is (token, kv head, chunk) with chunks = clamp(G / (tokens * kv heads), 1, MK_ATTN_MAX_CHUNKS): never
      // more than max(G, tokens * kv heads) units, each holding q/kv head partials
      const size_t units = (size_t)std::max(g->G, rt.max_tokens * s.num_kv_heads);
      const int qpk = s.num_q_heads / s.num_kv_heads;
      if ((rc = dev_alloc(g, &p, units * qpk * MK_ATTN_PSTRIDE * sizeof(float), false))) return rc;
      s.aux0 = p;
      s.aux1 = rt.attn_cnt + g->attn_cnt_n / 2;
    }
  if ((rc = pack_weights(g, true))) return rc;
  g->single_copy = (c.flags & MK_CFG_SINGLE_WEIGHT_COPY) && c.max_num_batched_tokens >= 2;
  rt.packed_only = g->single_copy ? 1 : 0;
  g->releasable.assign(g->tensors.size(), 0);
  g->row_major_bytes = 0;
  {
    // which attached tensors does a linear stage read in place, and which do other stages read?
    auto storage_ids = [&](int id, std::vector<int> &out) {
      if (id < 0) return;
      const Tensor &t = g->tensors[id];
      if (t.kind == T_SHUFFLED) out.insert(out.end(), t.sources.begin(), t.sources.end());
      else out.push_back(id);
    };
    std::vector<char> as_linear_weight(g->tensors.size(), 0), otherwise(g->tensors.size(), 0);
    for (size_t si = 0; si < g->stages.size(); si++) {
      if (g->stages[si].op != MK_OP_LINEAR || g->stage_weight[si] < 0) continue;
      // (the forms that stream the tile copy at every token count need whole 64-wide steps per wavefront: k % 256 == 0)
      if (g->single_copy && (!g->stages[si].wpack || (g->stages[si].k & 255)))
        return fail(MK_EUNSUPPORTED, "MK_CFG_SINGLE_WEIGHT_COPY: the weight of stage %zu (%s) cannot be laid out in matrix-core tiles (k=%d is not a multiple of 256)", si,
                    g->stage_desc[si].c_str(), g->stages[si].k);
      std::vector<int> ids;
      storage_ids(g->stage_weight[si], ids);
      for (int id : ids) as_linear_weight[id] = 1;
    }
    // every other use of a tensor: any operand of any task except the weight operand (the second) of a linear task
    for (const Task &t : g->ltasks) {
      bool r_, s_;
      int e_;
      const bool lin = linear_kind(t.name, &r_, &s_, &e_) || t.name == "silu_mul_linear_with_residual";
      for (size_t a = 0; a < t.ops.size(); a++) {
        if (t.ops[a] < 0 || (lin && a == 1)) continue;
        std::vector<int> ids;
        storage_ids(t.ops[a], ids);
        for (int k : ids) otherwise[k] = 1;
      }
    }
    // the same memory attached under two ids (tied embedding / LM head) is in use as long as one of them is
    for (size_t a = 0; a < g->tensors.size(); a++)
      for (size_t b = 0; b < g->tensors.size(); b++)
        if (a != b && g->tensors[a].ptr && g->tensors[a].ptr == g->tensors[b].ptr && otherwise[b]) otherwise[a] = 1;
    for (size_t id = 0; id < g->tensors.size(); id++) {
      const Tensor &t = g->tensors[id];
      if (!as_linear_weight[id] || t.kind != T_ATTACHED) continue;
      if (g->single_copy && !otherwise[id]) g->releasable[id] = 1;
      else g->row_major_bytes += (int64_t)t.elems() * (int64_t)dtype_size(t.dtype);
    }
  }
  if ((rc = dev_alloc(g, &p, sizeof(MkStage) * (g->stages.size() + 1)))) return rc;
  g->d_stages = (MkStage *)p;
  rt.stages = g->d_stages;
  if (!g->stages.empty()) HIP_TRY(hipMemcpy(g->d_stages, g->stages.data(), sizeof(MkStage) * g->stages.size(), hipMemcpyHostToDevice));
  if ((rc = dev_alloc(g, &p, (size_t)g->G * 4 * 4 * 4 * 64 * 16, false))) return rc;
  rt.splitk_part = p;
  if ((rc = dev_alloc(g, &p, (size_t)g->G * 32 * sizeof(unsigned)))) return rc;
  rt.splitk_cnt = (unsigned *)p;
  g->timing_cap = 8192;
  if ((rc = dev_alloc(g, &p, sizeof(long long) * (g->timing_cap + 2)))) return rc;
  rt.timing = g->d_timing = (long long *)p;
  rt.timing_cap = g->timing_cap;
  if ((rc = dev_alloc(g, &p, sizeof(long long) * MK_PROF_TICKS * (g->stages.size() + 1) * g->G))) return rc;
  rt.stage_prof = (long long *)p;
  if ((rc = dev_alloc(g, &p, sizeof(unsigned) * (size_t)g->G))) return rc;
  rt.profiler_count = (unsigned *)p;
  rt.profiler = (unsigned long long *)g->profiler_ptr;
  rt.profiler_cap = g->profiler_cap;
  if ((rc = dev_alloc(g, &p, sizeof(MkRuntime)))) return rc;
  g->d_rt = (MkRuntime *)p;
  if ((rc = upload_runtime(g))) return rc;
  HIP_TRY(hipEventCreate(&g->ev0));
  HIP_TRY(hipEventCreate(&g->ev1));
  if ((rc = resolve_scratch(g->cfg.device))) return rc;  // set-up is where the static launch scratch's address is looked up
  g->compiled = true;
  return mk_init_requests(g);
}

int mk_init_requests(mk_graph *g) {
  if (!g || !g->compiled) return fail(MK_ESTATE, "mk_compile has not been called");
  if (g->launch_pending) return fail(MK_ESTATE, "a launch is still pending");
  HIP_TRY(hipSetDevice(g->cfg.device));
  const MkRuntime &rt = g->h_rt;
  HIP_TRY(hipDeviceSynchronize());
  HIP_TRY(hipMemset(rt.step, 0, sizeof(int) * rt.total_requests));
  HIP_TRY(hipMemset(rt.request_ids, 0xFF, sizeof(int) * rt.max_requests));
  if (rt.state_ids) {
    std::vector<int> ids(rt.max_requests);
    for (int i = 0; i < rt.max_requests; i++) ids[i] = i;
    HIP_TRY(hipMemcpy(rt.state_ids, ids.data(), sizeof(int) * rt.max_requests, hipMemcpyHostToDevice));
  }
  HIP_TRY(hipMemset(rt.qo_indptr, 0, sizeof(int) * (rt.max_requests + 1)));
  HIP_TRY(hipMemset(rt.kv_indptr, 0, sizeof(int) * (rt.max_requests + 1)));
  std::vector<int> pq(rt.max_pages);
  for (int i = 0; i < rt.max_pages; i++) pq[i] = i;
  HIP_TRY(hipMemcpy(rt.page_queue, pq.data(), sizeof(int) * rt.max_pages, hipMemcpyHostToDevice));
  MkSched sc;
  memset(&sc, 0, sizeof(sc));
  sc.page_queue_head = 0;
  sc.page_queue_tail = rt.max_pages;
  HIP_TRY(hipMemcpy(g->d_sched, &sc, sizeof(sc), hipMemcpyHostToDevice));
  HIP_TRY(hipMemset(rt.attn_cnt, 0, sizeof(unsigned) * g->attn_cnt_n));
  HIP_TRY(hipMemset(rt.splitk_cnt, 0, sizeof(unsigned) * 32 * (size_t)g->G));
  HIP_TRY(hipMemset(rt.profiler_count, 0, sizeof(unsigned) * (size_t)g->G));
  if (rt.profiler) HIP_TRY(hipMemset(rt.profiler, 0, sizeof(unsigned long long) * (size_t)rt.profiler_cap));
  return MK_OK;
}

int mk_set_profiler(mk_graph *g, void *device_u64, int64_t num_entries) {
  if (!g) return fail(MK_EINVAL, "null argument");
  if (g->launch_pending) return fail(MK_ESTATE, "a launch is still pending");
  if (device_u64 && num_entries < 2) return fail(MK_EINVAL, "a profiler tensor needs at least two entries");
  g->profiler_ptr = device_u64;
  g->profiler_cap = device_u64 ? num_entries : 0;
  if (g->compiled) {
    HIP_TRY(hipSetDevice(g->cfg.device));
    g->h_rt.profiler = (unsigned long long *)device_u64;
    g->h_rt.profiler_cap = g->profiler_cap;
    HIP_TRY(hipMemset(g->h_rt.profiler_count, 0, sizeof(unsigned) * (size_t)g->G));
    if (device_u64) HIP_TRY(hipMemset(device_u64, 0, sizeof(unsigned long long) * (size_t)num_entries));
    return upload_runtime(g);
  }
  return MK_OK;
}

int mk_enqueue_steps(mk_graph *g, void *stream, int max_iterations) {
  if (!g) return fail(MK_EINVAL, "null argument");
  if (max_iterations < 1) return fail(MK_EINVAL, "max_iterations must be positive");
  switch (g->cfg.mode) {
    case MK_MODE_OFFLINE: return do_launch(g, (hipStream_t)stream, max_iterations, MK_SCHED_OFFLINE);
    case MK_MODE_ONLINE: return do_launch(g, (hipStream_t)stream, max_iterations, MK_SCHED_ONLINE);
    default: return do_launch(g, (hipStream_t)stream, 1, MK_SCHED_FROM_META);  // the host's batch is run once
  }
}

int mk_enqueue_steps_static(mk_graph *g, void *stream, int max_iterations) {
  if (!g) return fail(MK_EINVAL, "null argument");
  if (!g->compiled) return fail(MK_ESTATE, "mk_compile has not been called");
  if (max_iterations < 1) return fail(MK_EINVAL, "max_iterations must be positive");
  if (g->G > MK_STATIC_MAX_WG) return fail(MK_EINVAL, "the static launch scratch holds %d workgroups, this graph runs %d", MK_STATIC_MAX_WG, g->G);
  if (g->h_rt.max_tokens * g->max_kv_heads > MK_STATIC_MAX_ITEMS || g->max_qpk > MK_STATIC_MAX_QPK)
    return fail(MK_EINVAL, "the static launch scratch holds %d (token, kv head) pairs of up to %d q heads each; this graph needs %d x %d",
                MK_STATIC_MAX_ITEMS, MK_STATIC_MAX_QPK, g->h_rt.max_tokens * g->max_kv_heads, g->max_qpk);
  if (g->flex_items > (size_t)MK_STATIC_MAX_ITEMS || g->flex_part > MK_STATIC_ATTN_HEADS * MK_ATTN_PSTRIDE)
    return fail(MK_EINVAL, "the static launch scratch is too small for this graph's attention stages (%zu work items)", g->flex_items);
  int rc = resolve_scratch(g->cfg.device);  // already resolved by mk_compile on this device; no allocation either way
  if (rc) return rc;
  if (g->launch_pending) return fail(MK_ESTATE, "a launch is still pending: call mk_wait first");
  HIP_TRY(hipSetDevice(g->cfg.device));
  unsigned char *base = g_scratch_ptr[g->cfg.device];
  MkRuntime rt = g->h_rt;
  rt.sync = (MkSync *)(base + SS_SYNC);
  rt.splitk_cnt = (unsigned *)(base + SS_SPLITK_CNT);
  rt.attn_cnt = (unsigned *)(base + SS_ATTN_CNT);
  rt.argmax_pv = (float *)(base + SS_ARGMAX_PV);
  rt.argmax_pi = (int *)(base + SS_ARGMAX_PI);
  rt.attn_part = (float *)(base + SS_ATTN_PART);
  rt.splitk_part = base + SS_SPLITK_PART;
  rt.stage_prof = nullptr;  // per-stage timing is library-allocated scratch too: not recorded by this entry point
  rt.timing = nullptr;
  // the array keeps what the previous call left: barrier state and arrival counters must start at zero
  hipLaunchKernelGGL(mk_fill_zero_kernel, dim3(16), dim3(256), 0, (hipStream_t)stream, (uint4 *)base, SS_CLEARED_END / 16);
  HIP_TRY(hipGetLastError());
  const int sched = g->cfg.mode == MK_MODE_OFFLINE ? MK_SCHED_OFFLINE : (g->cfg.mode == MK_MODE_ONLINE ? MK_SCHED_ONLINE : MK_SCHED_FROM_META);
  return do_launch(g, (hipStream_t)stream, sched == MK_SCHED_FROM_META ? 1 : max_iterations, sched, &rt, true);
}

int mk_wait(mk_graph *g, void *stream, int *finished_out) {
  if (!g) return fail(MK_EINVAL, "null argument");
  return do_wait(g, (hipStream_t)stream, finished_out);
}

int mk_launch_steps(mk_graph *g, void *stream, int max_iterations, int *finished_out) {
  int rc = mk_enqueue_steps(g, stream, max_iterations);
  if (rc) return rc;
  return mk_wait(g, stream, finished_out);
}

int mk_launch(mk_graph *g, void *stream) {
  int finished = 0;
  int rc = mk_launch_steps(g, stream, 0x7fffffff, &finished);
  if (rc) return rc;
  const bool runs_to_completion = g->cfg.mode == MK_MODE_OFFLINE || g->cfg.mode == MK_MODE_ONLINE;
  if (runs_to_completion && !finished) return fail(MK_EABORT, "kernel returned before all requests finished");
  return MK_OK;
}

int mk_run_once(mk_graph *g, void *stream, int num_tokens, const int32_t *tok_slot, const int32_t *tok_pos, const int32_t *tok_first) {
  if (!g || !g->compiled) return fail(MK_ESTATE, "mk_compile has not been called");
  const MkRuntime &rt = g->h_rt;
  if (num_tokens < 1 || num_tokens > rt.max_tokens) return fail(MK_EINVAL, "num_tokens=%d outside [1, %d]", num_tokens, rt.max_tokens);
  if (!tok_slot || !tok_pos || !tok_first) return fail(MK_EINVAL, "null argument");
  for (int t = 0; t < num_tokens; t++) {
    if (tok_slot[t] < 0 || tok_slot[t] >= rt.max_requests) return fail(MK_EINVAL, "tok_slot[%d]=%d out of range", t, tok_slot[t]);
    if (tok_pos[t] < 0 || tok_pos[t] >= rt.max_seq) return fail(MK_EINVAL, "tok_pos[%d]=%d outside [0, max_seq_length)", t, tok_pos[t]);
    if (tok_first[t] < 0 || tok_first[t] > t || tok_slot[tok_first[t]] != tok_slot[t] || tok_pos[t] - tok_pos[tok_first[t]] != t - tok_first[t] ||
        t - tok_first[t] >= rt.max_new_per_req)
      return fail(MK_EINVAL, "tok_first[%d]=%d is not the first row of a contiguous run of <= %d tokens of the same request", t, tok_first[t], rt.max_new_per_req);
  }
  HIP_TRY(hipSetDevice(g->cfg.device));
  hipStream_t s = (hipStream_t)stream;
  HIP_TRY(hipStreamSynchronize(s));
  HIP_TRY(hipMemcpy(rt.tok_slot, tok_slot, sizeof(int) * num_tokens, hipMemcpyHostToDevice));
  HIP_TRY(hipMemcpy(rt.tok_pos, tok_pos, sizeof(int) * num_tokens, hipMemcpyHostToDevice));
  HIP_TRY(hipMemcpy(rt.tok_first, tok_first, sizeof(int) * num_tokens, hipMemcpyHostToDevice));
  MkSched sc;
  HIP_TRY(hipMemcpy(&sc, g->d_sched, sizeof(sc), hipMemcpyDeviceToHost));
  sc.num_tokens = num_tokens;
  sc.bad_batch = 0;
  HIP_TRY(hipMemcpy(g->d_sched, &sc, sizeof(sc), hipMemcpyHostToDevice));
  int rc = do_launch(g, s, 1, MK_SCHED_HOST_ARRAYS);
  if (rc) return rc;
  return do_wait(g, s, nullptr);
}

int mk_get_stats(mk_graph *g, mk_stats *out) {
  if (!g || !out) return fail(MK_EINVAL, "null argument");
  memset(out, 0, sizeof(*out));
  out->num_workgroups = g->G;
  out->num_stages = (int)g->stages.size();
  out->num_tasks = g->num_ref_tasks;
  out->num_events = g->num_ref_events;
  out->num_xcds = g->last_nxcd;
  out->aborted = g->last_aborted;
  out->weight_bytes = g->weight_bytes;
  out->packed_weight_bytes = g->packed_bytes;
  out->row_major_weight_bytes = g->row_major_bytes;
  out->last_launch_ms = g->last_ms;
  if (g->compiled && !g->launch_pending) {
    MkSched sc;
    HIP_TRY(hipMemcpy(&sc, g->d_sched, sizeof(sc), hipMemcpyDeviceToHost));
    out->iterations = sc.iterations;
  }
  return MK_OK;
}

// ticks [first, first + 4) of the stage records of one workgroup, scheduler record last
static int copy_stage_ticks(mk_graph *g, int workgroup, int first, int64_t *ticks_out, int max_stages) {
  if (!g || !ticks_out) return fail(MK_EINVAL, "null argument");
  if (!g->compiled || g->launch_pending) return fail(MK_ESTATE, "no finished launch to report");
  if (workgroup < 0 || workgroup >= g->G) return fail(MK_EINVAL, "workgroup %d outside [0, %d)", workgroup, g->G);
  const int recs = (int)g->stages.size() + 1;
  const int n = std::min<int>(max_stages, recs);
  if (n <= 0) return 0;
  std::vector<long long> buf((size_t)MK_PROF_TICKS * recs);
  HIP_TRY(hipMemcpy(buf.data(), g->h_rt.stage_prof + (size_t)MK_PROF_TICKS * workgroup * recs, sizeof(long long) * buf.size(), hipMemcpyDeviceToHost));
  for (int s = 0; s < n; s++)
    for (int k = 0; k < 4; k++) ticks_out[4 * s + k] = buf[(size_t)MK_PROF_TICKS * s + first + k];
  return n;
}

int mk_get_stage_profile(mk_graph *g, int workgroup, int64_t *ticks_out, int max_stages) { return copy_stage_ticks(g, workgroup, 0, ticks_out, max_stages); }

int mk_get_stage_marks(mk_graph *g, int workgroup, int64_t *ticks_out, int max_stages) { return copy_stage_ticks(g, workgroup, 4, ticks_out, max_stages); }

int mk_describe_program(mk_graph *g, const char **text_out) {
  if (!g || !text_out) return fail(MK_EINVAL, "null argument");
  if (!g->compiled) {
    int rc = lower(g);
    if (rc) return rc;
  }
  *text_out = g->program_text.c_str();
  return MK_OK;
}

}  // extern "C"
