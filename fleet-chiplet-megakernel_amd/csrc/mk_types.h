// Descriptors shared between the host lowering (mk_host.cpp) and the persistent
// decode megakernel (mk_kernel.hip).  Everything here is plain-old-data that is
// copied to HBM once at compile() time; the kernel is data-driven and never
// recompiled per model.
//
// Role in the reference: these structs take the place of TaskDesc / EventDesc /
// RuntimeConfig (include/mirage/persistent_kernel/runtime_header.h:200-375), but
// describe a *stage program* (one entry per fused operator, statically tiled
// over the workgroups of the 8 XCDs) instead of per-tile tasks in queues.
#pragma once
#include <stdint.h>

#ifdef __HIP__
#define MK_HOST_DEVICE __host__ __device__
#else
#define MK_HOST_DEVICE
#endif

#define MK_THREADS 256        // threads per workgroup (4 wavefronts of 64)
#define MK_WAVES 4
#define MK_MAX_XCD 16
#define MK_MAX_SEGS 3         // a shuffled weight has at most 3 sources (q,k,v)
#define MK_MAX_TOKENS 64      // max tokens per iteration supported by the kernels
#define MK_ATTN_MAX_CHUNKS 32 // split-KV fan-out limit per (token, kv head)
#define MK_ATTN_PSTRIDE 160   // floats per (work unit, q head) split-KV partial: 128 values + one 128-byte line of (max, sum)
#define MK_MAX_NEW_PER_REQ 64 // most prompt tokens one request may ingest per iteration (the attention stage keeps their K/V rows in LDS); the
#define MK_ATTN_MAX_REQ_PAGES 8192  // page-table entries of one request the attention stage keeps in LDS: max_seq_length / page_size may not exceed it
                              // configured value defaults to the reference's 8 (MPK_MAX_TOKENS_PER_REQUEST, persistent_kernel.cuh:115-124)
// LDS map of one workgroup (dynamic, > 80 KB pins one workgroup per CU):
//   [0, 24 KB)      input row(s) of the running stage / attention scratch (attention may run on beyond 32 KB)
//   [24 KB, 25 KB)  reduction scratch
//   [25 KB, 32 KB)  outputs of a single-token linear, collected before they are written out
//   [32 KB, 128 KB) routing lists of the mixture-of-experts stages, matrix-core reduction scratch
//   the matrix-core linear that keeps its token rows resident uses [0, 128 KB) for them and the words above for its flags
// (gfx950 gives a workgroup up to 160 KB; 156 KB dynamic + the kernel's static arrays stay below that)
#define MK_RED_OFFSET (24 * 1024)
#define MK_OUT_OFFSET (25 * 1024)   // [25 KB, 32 KB): outputs of a single-token linear collected before they are written out
#define MK_MOE_OFFSET (32 * 1024)
#define MK_MOE_X_OFFSET (40 * 1024)  // [40 KB, 128 KB): input rows of a multi-token MoE linear's (token, slot) pairs
#define MK_LDS_BYTES (156 * 1024)
#define MK_PROF_TICKS 8

enum MkOp {
  MK_OP_NONE = 0,
  MK_OP_EMBED = 1,
  MK_OP_NORM = 2,
  MK_OP_LINEAR = 3,
  MK_OP_SILU_MUL = 4,
  MK_OP_ATTN = 5,
  MK_OP_ARGMAX_PARTIAL = 6,
  MK_OP_ARGMAX_REDUCE = 7,
  MK_OP_MOE_TOPK = 8,     // router softmax -> top-k -> renormalise, one wavefront per token
  MK_OP_MOE_LINEAR = 9,   // per-expert linear over the active experts (W13 with optional SwiGLU, W2)
  MK_OP_MOE_COMBINE = 10, // out = res + sum_k w[t,k] * x[t,k,:]
  MK_OP_COPY = 11,        // out[t, :] = in[t, :], n 16-bit units per token row
  // prompt-lookup speculative decoding (integer stages; tasks/speculative_decoding/prompt_lookup.cuh, target_verify.cuh)
  MK_OP_NGRAM_PARTIAL = 12,  // out[slot, task] = earliest position among the task's share where the request's last k tokens occurred before
  MK_OP_NGRAM_GLOBAL = 13,   // out[row] = this iteration's token ids: the scheduler's, and for a decoding request the tokens after that position
  MK_OP_VERIFY = 14,         // num_new_tokens[request] = 1 + leading candidates the sampled tokens agree with
  // stages whose sizes and constants are data (mk_flex.hip); a graph that holds one runs on the flex kernels
  MK_OP_FX_EMBED = 15,       // out2 = table[id] * alpha in 32 bits, out = the same rounded
  MK_OP_FX_ADDNORM = 16,     // v = alpha * res + in; out2 = v / rms(v) * (w_offset + w) in 32 bits, out = the same rounded
  MK_OP_FX_PREP = 17,        // rotate / normalise q and k rows, append K/V (iterations in which a request brings several tokens)
  MK_OP_FX_ATTN = 18,        // paged attention with softcap and sink (single-token iterations: preparation and append included)
  MK_OP_LINEAR_F32 = 19,     // LINEAR with 32-bit operands
  MK_OP_FX_ARGMAX_F32 = 20,  // ARGMAX_PARTIAL over 32-bit logits
  // latent attention, recurrence and what goes with them (mk_mix.hip); a graph that holds one runs on the mix kernels
  MK_OP_MX_PRENORM = 21,     // v = res + alpha * in (in: optionally RMS-normalised first); out2 = v in 32 bits, out = group RMS norm of v (or v), rounded
  MK_OP_MX_LATENT_PREP = 22, // normalised query latents, normalised + rotated key latents into their pages, gated activation
  MK_OP_MX_HEAD_LINEAR = 23, // one small matrix per head; optionally gelu(...) * a per-token table row
  MK_OP_MX_LATENT_ATTN = 24, // attention in the latent space, one shared key/value row per position
  MK_OP_MX_LATENT_MERGE = 25,  // chunks of the latent attention (iterations in which some request was split)
  MK_OP_MX_DECAY = 26,       // decays of the delta rule (low-rank product of tanh), gated activation beside it
  MK_OP_MX_DELTA = 27,       // generalised delta rule: recurrent state per request and head
  MK_OP_MX_DELTA_OUT = 28,   // norm and gate of its outputs (iterations that dealt heads in slices)
  // selective scan, expert feed-forwards (mk_hybrid.hip); a graph that holds one, or a linear / attention / norm stage with an
  // option of theirs, runs on the hybrid kernels
  MK_OP_HY_CONV = 29,        // causal convolution per channel + silu
  MK_OP_HY_STEP = 30,        // HEAD_LINEAR with a softplus behind an offset, 32-bit result (step sizes of the scan)
  MK_OP_HY_SCAN = 31,        // selective scan: recurrent state per request, channel and state; convolution tail
  MK_OP_HY_ROUTE = 32,       // router softmax -> top-k -> renormalise over 32-bit logits (iterations of several tokens)
  MK_OP_HY_EXPERTS = 33,     // expert linears over the routed tokens and a shared expert over all of them
  // parallel sub-layers, state-space recurrence with one decay per head (mk_dual.hip); a graph that holds one, or an older stage
  // with an option of theirs, runs on the dual kernels
  MK_OP_DU_CONV = 34,        // causal convolution per channel whose inputs stay in a ring of rows per request; step sizes and decays beside it
  MK_OP_DU_SCAN = 35,        // recurrence per head, [states x values] of state, gated 32-bit result
};

enum MkStageFlags {
  MK_F_NORM = 1,         // LINEAR: RMSNorm(in, norm_w) is applied to the input rows
  MK_F_RES = 2,          // LINEAR: out = acc + res
  MK_F_SILU = 4,         // LINEAR: weight rows interleave [gate ; up]; out = silu(gate)*up
  MK_F_QK_NORM = 8,      // ATTN: per-head RMSNorm on q and k
  MK_F_ROPE = 16,        // ATTN: rotate-half RoPE on q and k
  MK_F_ONLY_MULTI = 32,  // stage runs only when the iteration has more than one token
  MK_F_EMBED_FROM_TOKENS = 64,  // EMBED: ids come from tokens[req, step+j] instead of input_tokens
  MK_F_MOE_INLINE_TOPK = 128,   // MOE_LINEAR: a single-token iteration routes inside this stage (the MOE_TOPK stage before it is multi-token only)
  MK_F_MOE_COMBINE = 256,       // MOE_LINEAR: a single-token iteration also forms res + sum_k w_k * y_k (the MOE_COMBINE stage after it is multi-token only)
  MK_F_DEFER_SUM = 512,  // LINEAR: the next stage is a full-row NORM over this stage's output, which may be handed the K-slice partials to sum
  MK_F_ADDNORM = 1024,   // LINEAR (set together with MK_F_NORM): the norm in front is an FX_ADDNORM; a single-token iteration forms it inside this stage
  MK_F_PRENORM = 4096,   // LINEAR (set together with MK_F_NORM): the norm in front is an MX_PRENORM; a single-token iteration forms it inside this stage
  MK_F_GELU_TABLE = 8192,  // MX_HEAD_LINEAR: out = gelu(acc) * table[id][n]
  MK_F_JOIN = 16384,     // LINEAR: a single-token iteration adds the result to the residual stream itself (the MX_PRENORM behind is multi-token only)
  MK_F_RELU2 = 32768,    // LINEAR: out = max(acc, 0)^2
  MK_F_OUT32 = 65536,    // MX_HEAD_LINEAR: 32-bit result in out2
  MK_F_GELU = 131072,    // with MK_F_SILU: the gate is gelu (tanh form) instead of silu
  MK_F_CLAMP_GLU = 262144,  // with MK_F_SILU, HY_EXPERTS: out = a / (1 + exp(-beta a)) * (b + bias), a = min(gate, limit), b = clamp(up, -limit, limit)
  MK_F_GROUPS = 524288,  // HY_ROUTE / HY_EXPERTS: sigmoid scores, choice with a correction among the best groups of experts
  MK_F_ROW_NORM = 1048576,  // FX_ATTN / FX_PREP: all query heads of a row are RMS-normalised together, all key heads likewise
  MK_F_PORTIONS = 2097152,  // DU_CONV: iterations in which some request brings several tokens (the norm in front does it otherwise)
  MK_F_IDENTITY = 4194304,  // DU_CONV: the input itself is added
  MK_F_RES_EARLY = 2048, // FX_ADDNORM / LINEAR+ADDNORM: the stage before this one does not write the residual rows, so they may be requested before its barrier
};

#define MK_MX_MAX_GROUPS 256     // parts of a row with a norm of their own
#define MK_MX_MAX_NORM_ROW 4096  // longest query latent / key latent row a wavefront normalises
#define MK_MX_MAX_LATENT 512     // key latent size of the latent attention
#define MK_MX_MAX_CHUNKS 64      // split of a request's cached latents (one lane of the merging wavefront each)
#define MK_MX_MAX_DELTA_DIM 256  // head size of the recurrence
#define MK_MX_MAX_RANK 1024      // low-rank decay projection

#define MK_HY_MAX_STATES 256     // states per channel of the selective scan
#define MK_DU_MAX_TAPS 16        // taps of the convolutions that keep a ring of rows

#define MK_FX_MAX_HEAD_DIM 512  // largest q/k head the flex attention keeps in a wavefront's registers

#define MK_MOE_MAX_EXPERTS 256  // one thread per expert when the routing lists are built
#define MK_MOE_MAX_TOPK 16

// A (possibly shuffled) weight matrix [rows, k] bf16.  Virtual row r of a shuffled
// tensor lives in source `seg` at a row computed from the group structure, so no
// interleaved copy is ever made (the reference materialises one,
// src/kernel/runtime.cc:904-943).
struct MkWeight {
  const void *seg[MK_MAX_SEGS];
  int seg_rows[MK_MAX_SEGS];  // rows each source contributes to one group
  int nseg;
  int group_rows;  // sum of seg_rows (== total rows when nseg == 1)
  int pad0, pad1;
};

struct MkStage {
  int op;
  int flags;
  int n;  // LINEAR: virtual weight rows; ARGMAX: vocabulary; SILU_MUL: output columns
  int k;  // LINEAR: reduction length; NORM / EMBED: row length
  int ld_in, ld_out, ld_res, silu_half;  // leading dimensions in elements; silu_half = rows of gate per group
  float eps;
  int groups;  // SILU_MUL: number of [gate;up] groups
  const void *in;
  void *out;
  const void *res;
  const void *norm_w;
  void *norm_out;
  MkWeight w;
  // LINEAR: the same weights re-laid for the matrix cores (null: none), in 16-row tiles -- plain stages tile t = rows
  // [16 t, 16 t + 16), SwiGLU stages tile 2j = gate rows of outputs [16 j, 16 j + 16) and tile 2j + 1 their up rows --
  // as [tile][k / 64][2][64 lanes] 16-byte operands: lane l of (tile, step, h) holds k = 64 step + 32 h + 8 (l / 16) ..
  // + 7 of the tile's row l % 16.  A tile is one contiguous stream of 32 k bytes.
  const void *wpack;
  // attention
  void *k_cache, *v_cache;
  const void *q_norm_w, *k_norm_w, *cos_tab, *sin_tab;
  void *q_ws;
  int num_q_heads, num_kv_heads, head_dim, ld_qws;
  int ld_cos, ld_norm;  // ld_norm: leading dimension of norm_out
  float sm_scale_log2;  // log2(e) / sqrt(head_dim)
  int prof_event;       // the reference's task-type number this stage is recorded under in a caller's profiler tensor
  // argmax
  void *aux0, *aux1;
  // mixture of experts.  MOE_LINEAR: x(t,slot) = in + t*ld_in + slot*ld_in_slot, expert e's weights are rows
  // [e*n, (e+1)*n) of w.seg[0], y(t,slot,row) = out + t*ld_out + slot*ld_out_slot + row; with MK_F_SILU rows
  // [0,n/2) are gate and [n/2,n) up, and out2(t,slot,j) receives silu(gate_j)*up_j; with MK_F_MOE_COMBINE out2 is
  // the [tokens, n] result of the weighted sum.
  const void *moe_logits;  // [tokens, num_experts] bf16 router logits (ld_logits)
  float *moe_topk_w;       // [tokens, topk] fp32 renormalised routing weights (ld_topk_w)
  int *moe_routing;        // [num_experts, tokens] int32: 1 + top-k slot of the expert for that token, 0 = not routed
  int *moe_mask;           // [num_experts + 1] int32: ids of the active experts, then their count at [num_experts]
  void *out2;
  int num_experts, topk, ld_logits, ld_topk_w;
  int ld_routing, ld_in_slot, ld_out_slot, ld_out2;
  int ld_out2_slot;
  // flex stages (mk_flex.hip)
  int k_tiles, v_tiles;  // FX_ATTN: instantiation -- operand rows of a key / 16-wide value blocks held at a time
  int rot_dims;          // FX_ATTN: rotated dims of a head (head_dim: query/key size)
  // FX_ADDNORM and LINEAR+ADDNORM: rows are padded with zeros to `n` / `k` entries, `k` / `k_real` of them are real; y_in: the
  // rows added to alpha * res (null: none); out2: the 32-bit result.
  const void *y_in;
  const void *sink;      // FX_ATTN: [num_q_heads] fp32, null: none
  float alpha, w_offset; // residual (or embedding) factor; constant added to the norm weight
  float sm_scale, softcap;  // FX_ATTN: score factor, tanh cap (0: none)
  float norm_eps;        // LINEAR+ADDNORM: eps of the fused norm
  int k_real, ld_y;
  int v_dim;             // FX_ATTN: value size per head
  // mix stages (mk_mix.hip)
  const void *y_norm_w;  // MX_PRENORM / LINEAR+PRENORM: fp32 weight of the RMS norm of the summand (null: none)
  int norm_groups;       // ... parts of the output norm (0: no norm)
  int rank;              // key latent size (latent stages)
  int nk;                // MX_LATENT_ATTN: operand rows of a cached latent its instantiation holds
  int cols[5];           // columns of `in`: MX_LATENT_PREP q latent, k latent, rotated key part; MX_LATENT_ATTN rotated query part of a head; MX_DELTA r k v g a
  const void *in2;       // MX_DELTA: decays, 32-bit rows (out2 / ld_out2: unnormalised outputs)
  int ld_in2, pad_in2;
  // gated activation beside MX_LATENT_PREP / MX_DECAY: out = a / (1 + exp(-beta a)) * (b + bias), a = min(gate, limit), b = clamp(up, -limit, limit)
  void *glu_out;
  int glu_n, ld_glu, glu_gate, glu_up;
  float glu_limit, glu_beta, glu_bias;
  // hybrid stages (mk_hybrid.hip) and the options of older ones that go with them
  int window, keep_first;  // FX_ATTN: a position sees the `window` newest ones (0: all) and the `keep_first` first ones
  int v_col;               // FX_ATTN: column the value heads begin at
  int slots;               // MX_PRENORM / LINEAR+PRENORM: summands per row (0: one, unweighted); HY_EXPERTS: rows per token
  int ld_slot, ld_slot_w;  // ... columns per summand, weights per row
  const float *slot_w;     // ... fp32 [tokens, ld_slot_w]
  const float *in_bias;    // FX_ATTN / FX_PREP: added to the input rows; MX_PRENORM: added to the summand; HY_CONV; HY_STEP
  const void *w_shared;    // HY_EXPERTS: weights of the expert every token visits (null: none)
  int *ids;                // HY_ROUTE, HY_EXPERTS: int32 [tokens, topk] chosen experts
  int n_shared, k_shared;  // HY_EXPERTS: outputs and reduction length of the shared expert
  int states, taps;        // HY_SCAN: states per channel, taps of the convolution
  const float *a_tab, *d_tab;  // HY_SCAN: fp32 [channels, states] log2(e) * A, [channels]
  void *tail;              // HY_CONV / HY_SCAN: last inputs of the convolution, [state slot][taps - 1][channels]
  const void *in3;         // HY_SCAN: step / B / C rows
  int ld_in3;
  // dual stages (mk_dual.hip) and the options of older ones that go with them
  int chunk;               // FX_ATTN: a position sees only its own chunk of this many (0: no chunks)
  const float *temp;       // FX_ATTN: fp32 [num_q_heads] factor of the scores
  const float *y_scale;    // MX_PRENORM / LINEAR+PRENORM: fp32 factor of the summand, element by element (null: none)
  const void *y2;          // ... a second summand (null: none; `slots` then belongs to it) and its factor
  const float *y2_scale;
  const void *conv_w;      // ... and LINEAR: [taps][n] convolution over time of the normed rows, added to them: MX_PRENORM's out3, LINEAR's norm_out (ring: tail; LINEAR's out3: the normed rows); DU_CONV: its weights
  void *out3;
  const void *pos_tab;     // FX_EMBED: [pos_rows, k] added by position (null: none)
  int ld_y2, ld_out3, pos_rows, groups_keep;  // groups_keep: MK_F_GROUPS: groups (field `groups`) that stay open
  const float *choice_bias;  // MK_F_GROUPS: fp32 [num_experts] correction of the choice
  float choice_scale, glu_limit_shared;  // ... factor of the chosen scores; MK_F_CLAMP_GLU: limit of the shared expert
  const float *step_bias;  // DU_CONV: fp32 [num_q_heads] added to the step inputs (column cols[1]); rates in a_tab; steps and decays (column cols[2]) in out2
  int pad_du[4];
};
static_assert(sizeof(MkStage) % 64 == 0, "a descriptor is whole scalar-cache lines");

// LDS map of MX_LATENT_ATTN, in bytes: query operands, one tile of cached rows, weights of the tile's positions, row statistics,
// page-table entries.  RT: 16-row query tiles per unit; nkc: operand rows of a cached latent; sub: 16-position sub-tiles of a tile.
struct MkLatentLds {
  int kt, pb, mx, pages, bytes;
};
MK_HOST_DEVICE inline MkLatentLds mk_latent_lds(int es, int rt, int nkc, int sub, int max_pages) {
  MkLatentLds l;
  l.kt = rt * nkc * 1024;
  l.pb = l.kt + sub * nkc * 1024;
  l.mx = l.pb + rt * 1024 * (es == 2 ? (sub + 1) / 2 * 2 : sub);
  l.pages = l.mx + 2 * 4 * rt * 16 * 4;
  l.bytes = l.pages + (max_pages + 1) * 4;
  return l;
}

// Hierarchical barrier state.  One 128-byte line per counter so that XCD-local
// counters stay in that XCD's L2.
struct MkSync {
  unsigned global_ctr;
  unsigned pad0[31];
  unsigned local_ctr[MK_MAX_XCD][32];
  unsigned local_flag[MK_MAX_XCD][32];
  unsigned xcd_count[MK_MAX_XCD];
  unsigned pad1[32 - MK_MAX_XCD];
  unsigned init_ctr;
  unsigned pad2[31];
  unsigned abort_flag;
  unsigned abort_where;
  unsigned pad3[30];
};

// Barrier completion test.  Arrival counters and their targets (quota x epoch) are 32-bit and only ever grow during a
// launch, so on a long launch both wrap; their difference taken as a signed number stays correct as long as the two
// are less than 2^31 apart, and they are never more than one stage apart.
MK_HOST_DEVICE inline bool mk_counter_reached(unsigned counter, unsigned target) { return (int)(counter - target) >= 0; }

// Who describes the batch of an iteration (the kernel's `run_scheduler` argument).
enum MkSchedMode {
  MK_SCHED_HOST_ARRAYS = 0,  // the host wrote tok_slot / tok_pos / tok_first (mk_run_once)
  MK_SCHED_OFFLINE = 1,      // on-GPU continuous batching over `tokens` (MODE_OFFLINE)
  MK_SCHED_FROM_META = 2,    // derived on the GPU from the qo / paged-kv meta tensors the host filled (MODE_ONLINE_NOTOKEN, MODE_ONEPASS)
  MK_SCHED_ONLINE = 3,       // one request, host-written tokens consumed num_new_tokens[0] at a time (MODE_ONLINE)
};

// Scheduler state that persists across launches (continuous batching, page ring).
struct MkSched {
  int page_queue_head, page_queue_tail, next_request_id, num_tokens;
  int num_reqs, finished, online_started;
  int bad_batch;          // host-described batch (MK_SCHED_FROM_META) that was rejected instead of run: 0 = fine, else the reason

  long long iterations;   // decode iterations executed so far (all launches)
  long long pad2;
};

struct MkRuntime {
  int num_stages, max_tokens, max_requests, max_seq;
  int page_size, max_pages, total_requests, max_new_per_req;
  int spec_len, pad_spec;  // speculative candidates a decoding request brings into an iteration beside its newest token (0: none)
  long long eos_token_id;
  // meta tensors (persistent_kernel.py:2590-2600 order)
  int *step;
  long long *tokens;
  long long *input_tokens;
  long long *output_tokens;
  int *num_new_tokens;
  int *prompt_lengths;
  int *qo_indptr;
  int *kv_indptr;
  int *kv_indices;
  int *kv_last_page_len;
  // library-owned scheduler memory
  int *request_ids;   // [max_requests] request id per batch slot, -1 = free
  int *state_ids;     // [max_requests] recurrent-state slot per batch slot, a permutation (null: the graph has no recurrence)
  int *page_queue;    // [max_pages] ring of free page ids
  int *tok_slot;      // [max_tokens] batch slot of each token of this iteration
  int *tok_pos;       // [max_tokens] absolute position of each token
  int *tok_first;     // [max_tokens] index of the first token of the same request in this iteration
  MkSched *sched;
  const MkStage *stages;
  MkSync *sync;
  // attention split-KV workspace
  float *attn_part;     // null: every attention stage has a partial buffer of its own (its descriptor's aux0).  Non-null: ONE buffer
                        // [units][q/kv][MK_ATTN_PSTRIDE] shared by all attention stages, handed off at device scope only
  float *argmax_pv;     // non-null: the sampling stages' per-workgroup partials live here ([tokens][workgroups] values / indices)
  int *argmax_pi;       // instead of in the buffers their descriptors name
  unsigned *attn_cnt;   // [max_tokens * num_kv_heads][32]: one 128-byte line per counter
  void *splitk_part;    // [workgroups][4 wavefronts][4 weight tiles][4 token tiles][64 lanes] f32x4: K-slice partials of the split-K linear
  unsigned *splitk_cnt; // [workgroups][32]: arrival counter per split-K group (one 128-byte line each)
  long long *timing;    // [1 + timing_cap] wall-clock ticks (100 MHz) at the start of each iteration; [0] = kernel end
  int timing_cap;
  int packed_only;       // the handle keeps ONLY the matrix-core copies of its linear weights: iterations of one or two tokens run the matrix-core forms too
  // A caller's profiler tensor (null: none): (tag, time) entries of EVERY executed stage of every iteration, in the
  // reference's layout (include/mirage/persistent_kernel/profiler.h:129-180): entry 0 = (workgroups, 1); the k-th entry of
  // workgroup b sits at 1 + b + k * workgroups; low word tag = stage instance << 19 | b << 11 | task type << 2 | (0 begin, 1
  // end), high word = low 32 bits of the time in ns.  Recording stops when the tensor is full.
  unsigned long long *profiler;
  long long profiler_cap;        // entries the tensor holds
  unsigned *profiler_count;      // [workgroups] entries written so far by each workgroup (kept across launches)
  long long *stage_prof; // [workgroups][num_stages + 1][MK_PROF_TICKS] 100 MHz ticks of the last iteration: entry, wait done, exit, arrived, then
                         // four marks a stage may set in a build with MK_TRACE defined; the extra record holds the scheduler step:
                         // [0] previous iteration complete, [1] batch prepared, [2] batch published to every workgroup
};
