// Stages whose sizes and constants are all data (part of the persistent kernel, included by mk_kernel.hip).
//
// The stages above this file are written for one family of shapes (heads of 128 values, a bf16 residual stream, a norm
// in front of each sub-layer).  The ones here take any head size, separate value size and head grouping, keep the
// residual stream in 32 bits, and get every constant from their descriptor, so that a model of another design is another
// list of descriptors:
//   * stage_fx_embed    rows of a table times a constant, as 32-bit residual rows and as rows for the next linear;
//   * stage_fx_addnorm  alpha * x + y, RMS norm with weight (offset + w), written in both forms (y is optional);
//   * stage_fx_prep /   rotary positions on part of a head, heads divided by their root mean square, paged K/V append,
//     stage_fx_attn     softcapped scores, softmax with an extra per-head logit in the denominator, split-KV on the matrix
//                       cores for prompt portions and for single tokens alike;
//   * stage_fx_linear_f32, stage_fx_argmax_f32  the 32-bit forms of the linear and of the sampling stage.
// The stages are instantiated for bf16 (E = uint16_t) and for 32-bit (E = float) activations, weights and caches; scores,
// softmax, norms, angles and the residual stream are 32-bit in both.

template <typename E> struct FxType;
// EPC: elements per 16-byte operand; KW: head dims one matrix-core operand row covers (4 lane groups x EPC);
// TP: cached positions per tile; SUB: 16-position sub-tiles of a tile
template <> struct FxType<uint16_t> {
  static constexpr int EPC = 8, KW = 32, TP = 32, SUB = 2;
};
template <> struct FxType<float> {
  static constexpr int EPC = 4, KW = 16, TP = 16, SUB = 1;
};
__device__ __forceinline__ float fx_ldc(const uint16_t *p) { return bf2f(ldc_u16(p)); }
__device__ __forceinline__ float fx_ldc(const float *p) { return ldc_f32(p); }
__device__ __forceinline__ float fx_val(uint16_t v) { return bf2f(v); }
__device__ __forceinline__ float fx_val(float v) { return v; }
template <typename E> __device__ __forceinline__ E fx_round(float v) {
  if constexpr (sizeof(E) == 2) return (E)f2bf(v);
  else return v;
}
__device__ __forceinline__ void fx_stc(uint16_t *p, uint16_t v) { stc_u16(p, v); }
__device__ __forceinline__ void fx_stc(float *p, float v) { stc_f32(p, v); }
__device__ __forceinline__ void fx_stc4(uint16_t *row, int n0, int n_out, const float (&r)[4]) { stc_bf16x4(row, n0, n_out, r); }
__device__ __forceinline__ void fx_stc4(float *row, int n0, int n_out, const float (&r)[4]) {
#pragma unroll
  for (int i = 0; i < 4; i++)
    if (n0 + i < n_out) stc_f32(row + n0 + i, r[i]);
}
// four consecutive row elements, 16-byte (32-bit) or 8-byte (bf16) aligned
__device__ __forceinline__ f32x4 fx_ldc_quad(const uint16_t *p) {
  const unsigned long long u = ldc_u64(p);
  const uint32_t a = (uint32_t)u, b = (uint32_t)(u >> 32);
  return (f32x4){bf_lo(a), bf_hi(a), bf_lo(b), bf_hi(b)};
}
__device__ __forceinline__ f32x4 fx_ldc_quad(const float *p) { return __builtin_bit_cast(f32x4, ldc_16B((const u32x4 *)p)); }
// ... of a table nobody writes during a launch
__device__ __forceinline__ f32x4 fx_ld_quad(const uint16_t *p) {
  const unsigned long long u = *(const unsigned long long *)p;
  const uint32_t a = (uint32_t)u, b = (uint32_t)(u >> 32);
  return (f32x4){bf_lo(a), bf_hi(a), bf_lo(b), bf_hi(b)};
}
__device__ __forceinline__ f32x4 fx_ld_quad(const float *p) { return *(const f32x4 *)p; }
__device__ __forceinline__ void fx_stc_quad(uint16_t *p, f32x4 v) {
  stc_u64(p, (unsigned long long)pack2(v[0], v[1]) | ((unsigned long long)pack2(v[2], v[3]) << 32));
}
__device__ __forceinline__ void fx_stc_quad(float *p, f32x4 v) { stc_16B((u32x4 *)p, __builtin_bit_cast(u32x4, v)); }

// Maximum / sum over the four 16-lane groups of a wavefront (every lane gets the result of its column lane & 15).
__device__ __forceinline__ float groups_max(float v) {
  const unsigned u = __float_as_uint(v);
  const auto a = __builtin_amdgcn_permlane32_swap(u, u, false, false);
  v = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  const unsigned w = __float_as_uint(v);
  const auto b = __builtin_amdgcn_permlane16_swap(w, w, false, false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ __forceinline__ float groups_sum(float v) {
  const unsigned u = __float_as_uint(v);
  const auto a = __builtin_amdgcn_permlane32_swap(u, u, false, false);
  v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const unsigned w = __float_as_uint(v);
  const auto b = __builtin_amdgcn_permlane16_swap(w, w, false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// ----------------------------------------------------------------------------- embedding
// out2[t, :] = table[id] * alpha in 32 bits, out[t, :] = the same rounded to E.  A negative id gives a row of zeros.
template <typename E>
__device__ __forceinline__ void stage_fx_embed(CStage &st, Ctx &c, const MkRuntime &rt, int M) {
  barrier_wait(c);
  const int k = st.k;
  for (int t = c.vid; t < M; t += c.G) {
    long long id;
    if (st.flags & MK_F_EMBED_FROM_TOKENS) {
      const int req = ldc_i32(&rt.request_ids[ldc_i32(&rt.tok_slot[t])]);
      id = (long long)ldc_u64(&rt.tokens[(long long)req * rt.max_seq + ldc_i32(&rt.tok_pos[t])]);
    } else {
      id = (long long)ldc_u64((const long long *)st.in + t);
    }
    const float scale = id < 0 ? 0.f : st.alpha;
    const E *src = (const E *)st.w.seg[0] + (size_t)(id < 0 ? 0 : id) * k;
    E *out = (E *)st.out + (size_t)t * st.ld_out;
    float *out32 = st.out2 ? (float *)st.out2 + (size_t)t * st.ld_out2 : nullptr;
#if MK_HAVE_DUAL
    if (st.pos_tab) {  // (the caller keeps positions inside the table)
      const E *pos = (const E *)st.pos_tab + (size_t)min(c.sh_tok[t], st.pos_rows - 1) * k;
      if ((k & 3) == 0) {
        for (int i = threadIdx.x * 4; i < k; i += MK_THREADS * 4) {
          const f32x4 v = fx_ld_quad(src + i) * scale + fx_ld_quad(pos + i);
          if (out32) fx_stc_quad(out32 + i, v);
          fx_stc_quad(out + i, v);
        }
      } else {
        for (int i = threadIdx.x; i < k; i += MK_THREADS) {
          const float v = fmaf(fx_val(src[i]), scale, fx_val(pos[i]));
          if (out32) stc_f32(out32 + i, v);
          fx_stc(out + i, fx_round<E>(v));
        }
      }
      continue;
    }
#endif
    if ((k & 3) == 0) {
      for (int i = threadIdx.x * 4; i < k; i += MK_THREADS * 4) {
        f32x4 v;
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] = fx_val(src[i + e]) * scale;
        if (out32) fx_stc_quad(out32 + i, v);
        fx_stc_quad(out + i, v);
      }
    } else {
      for (int i = threadIdx.x; i < k; i += MK_THREADS) {
        const float v = fx_val(src[i]) * scale;
        if (out32) stc_f32(out32 + i, v);
        fx_stc(out + i, fx_round<E>(v));
      }
    }
  }
  c.wrote_through = true;
}

// ----------------------------------------------------------------------------- residual sum + RMS norm
// v = alpha * x + y;  out2 = v / sqrt(mean(v^2) + eps) * (w_offset + w) in 32 bits, out = the same rounded to E.  Rows are
// st.n long with st.k of them real (the rest is zero in every operand).  x (st.res) is 32-bit, y (st.in, null: none) is the
// preceding linear's output, or its K-slice partials when that linear left its sum to this stage.  A workgroup per row.
template <typename E, int NS>
__device__ __forceinline__ void stage_fx_addnorm_t(CStage &st, Ctx &c, int M, char *smem) {
  const int tid = threadIdx.x, n4 = st.n / 4;
  float *red = (float *)smem;
  const f32x4 *w4 = (const f32x4 *)st.norm_w;
  const float *xr = (const float *)st.res;
  const int t0 = c.even_xcds ? c.rank * c.nxcd + c.xi : c.vid;  // rows are dealt round-robin over the dies
  const bool early = st.flags & MK_F_RES_EARLY;
  f32x4 g[NS], x[NS];
  auto load_x = [&](int t) {
#pragma unroll
    for (int j = 0; j < NS; j++)
      if (j * MK_THREADS < n4) x[j] = fx_ldc_quad(xr + (size_t)t * st.ld_res + 4 * min(tid + j * MK_THREADS, n4 - 1));
  };
#pragma unroll
  for (int j = 0; j < NS; j++)
    if (j * MK_THREADS < n4) g[j] = w4[min(tid + j * MK_THREADS, n4 - 1)];
  // the residual row was written at least one barrier earlier than y: requested before the barrier is awaited (not by the
  // wavefront that polls it)
  const bool pre = early && t0 < M && tid >= 64;
  if (pre) load_x(t0);
  barrier_wait(c);
  const int dS = c.defer_S;
  c.defer_S = 0;
  const float *dpart = c.defer_part;
  const size_t dslice = (size_t)c.defer_rows * c.defer_n;
  for (int t = t0; t < M; t += c.G) {
    if (!(pre && t == t0)) load_x(t);
    float ss = 0.f;
    f32x4 v[NS];
#pragma unroll
    for (int j = 0; j < NS; j++)
      if (j * MK_THREADS < n4) {
        const int s = min(tid + j * MK_THREADS, n4 - 1);
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
        if (dS) {
          const float *p = dpart + (size_t)t * c.defer_n + 4 * s;
          auto sum_slices = [&](auto ns) {  // all slices requested at once, summed in slice order
            constexpr int Q = decltype(ns)::value;
            f32x4 q[Q];
#pragma unroll
            for (int b = 0; b < Q; b++) q[b] = fx_ldc_quad(p + b * dslice);
#pragma unroll
            for (int b = 0; b < Q; b++) y += q[b];
          };
          if (dS == 2) sum_slices(std::integral_constant<int, 2>{});
          else if (dS == 4) sum_slices(std::integral_constant<int, 4>{});
          else sum_slices(std::integral_constant<int, 8>{});
        } else if (st.in) {
          y = fx_ldc_quad((const E *)st.in + (size_t)t * st.ld_in + 4 * s);
        }
#pragma unroll
        for (int e = 0; e < 4; e++) v[j][e] = fmaf(st.alpha, x[j][e], y[e]);
      }
#pragma unroll
    for (int j = 0; j < NS; j++)
      if (j * MK_THREADS < n4) {
        const bool ok = tid + j * MK_THREADS < n4;
#pragma unroll
        for (int e = 0; e < 4; e++) ss += ok ? v[j][e] * v[j][e] : 0.f;
      }
    ss = block_sum(ss, red);
    const float r = 1.f / sqrtf(ss / (float)st.k + st.eps);
#pragma unroll
    for (int j = 0; j < NS; j++)
      if (tid + j * MK_THREADS < n4) {
        const int s = tid + j * MK_THREADS;
        f32x4 o;
#pragma unroll
        for (int e = 0; e < 4; e++) o[e] = (v[j][e] * r) * (st.w_offset + g[j][e]);
        if (st.out2) fx_stc_quad((float *)st.out2 + (size_t)t * st.ld_out2 + 4 * s, o);
        fx_stc_quad((E *)st.out + (size_t)t * st.ld_out + 4 * s, o);
      }
    __syncthreads();
  }
  c.wrote_through = true;
}
template <typename E>
__device__ __forceinline__ void stage_fx_addnorm(CStage &st, Ctx &c, int M, char *smem) {
  if (st.n <= 4 * 4 * MK_THREADS) stage_fx_addnorm_t<E, 4>(st, c, M, smem);
  else stage_fx_addnorm_t<E, 12>(st, c, M, smem);
}

// ----------------------------------------------------------------------------- head rows
// Where the q/k/v rows of an attention stage come from: the linear's output, or its unsummed K-slice partials.
template <typename E> struct FxRows {
  const E *in;
  int ld;
  int S;
  const float *part;
  size_t slice, ldp;
  const float *bias;  // (hybrid kernels) added to every row where it is used, null: none
  template <int NS> __device__ __forceinline__ float get(int tok, int col) const {
    if constexpr (NS == 0) {
      return fx_ldc(in + (size_t)tok * ld + col);
    } else {
      const float *p = part + (size_t)tok * ldp + col;
      float q[NS], s = 0.f;
#pragma unroll
      for (int b = 0; b < NS; b++) q[b] = ldc_f32(p + b * slice);
#pragma unroll
      for (int b = 0; b < NS; b++) s += q[b];
      return fx_val(fx_round<E>(s));
    }
  }
  // f(slices) with the slice count as a compile-time constant: one branch per row instead of one per element
  template <typename F> __device__ __forceinline__ void with_slices(F f) const {
    if (S == 0) f(std::integral_constant<int, 0>{});
    else if (S == 2) f(std::integral_constant<int, 2>{});
    else if (S == 4) f(std::integral_constant<int, 4>{});
    else f(std::integral_constant<int, 8>{});
  }
};
template <typename E> __device__ __forceinline__ FxRows<E> fx_rows(CStage &st, Ctx &c) {
  FxRows<E> r{(const E *)st.in, st.ld_in, c.defer_S, c.defer_part, (size_t)c.defer_rows * c.defer_n, (size_t)c.defer_n, MK_HAVE_HYB ? st.in_bias : nullptr};
  c.defer_S = 0;
  return r;
}
#define MK_FX_HEAD_REGS (MK_FX_MAX_HEAD_DIM / 64)
// One query or key head row by one wavefront: dims [0, rot) are rotated (dim i < rot / 2 pairs with i + rot / 2), then the
// row is divided by sqrt(mean(x^2) + eps) when the stage asks for it.  Split in a half that requests everything and a half
// that computes, so that a wavefront can have the requests of two rows in flight; put(d, value) for every d < D.
//
// Dual kernels, MK_F_ROW_NORM: the row's query heads (its key heads) are together divided by their root mean square and multiplied
// by a weight per column instead; `r` is that factor, `w` the weights.
struct FxHead {
  float x[MK_FX_HEAD_REGS], xp[MK_FX_HEAD_REGS], cs[MK_FX_HEAD_REGS], sn[MK_FX_HEAD_REGS];
#if MK_HAVE_HYB
  float b[MK_FX_HEAD_REGS], bp[MK_FX_HEAD_REGS];  // bias of x and xp
#endif
#if MK_HAVE_DUAL
  float r, w[MK_FX_HEAD_REGS];
#endif
};
#if MK_HAVE_DUAL
// Weights of the row norm for the head whose columns begin at `col`.
__device__ __forceinline__ void fx_row_weights(CStage &st, int col, int lane, FxHead &h) {
  if (!(st.flags & MK_F_ROW_NORM)) return;
  const int nq = st.num_q_heads * st.head_dim;
  const float *w = col < nq ? (const float *)st.q_norm_w + col : (const float *)st.k_norm_w + (col - nq);
#pragma unroll
  for (int j = 0; j < MK_FX_HEAD_REGS; j++)
    if (j * 64 < st.head_dim) h.w[j] = w[min(j * 64 + lane, st.head_dim - 1)];
}
// This lane's part of the sum of squares over columns [c0, c1) of a row, lane `id` of `n`.
template <typename E>
__device__ __forceinline__ float fx_row_squares(const E *row, int c0, int c1, int id, int n) {
  float ss = 0.f;
  for (int q0 = c0 / 4 + id; q0 * 4 < c1; q0 += 4 * n) {
    f32x4 v[4];
#pragma unroll
    for (int j = 0; j < 4; j++) v[j] = fx_ldc_quad(row + 4 * min(q0 + j * n, (c1 - 1) / 4));
#pragma unroll
    for (int j = 0; j < 4; j++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const int at = 4 * (q0 + j * n) + e;
        ss += at >= c0 && at < c1 ? v[j][e] * v[j][e] : 0.f;
      }
  }
  return ss;
}
#endif
// Bias of a row's columns (hybrid kernels): requested beside the row, added when it is used.
template <typename E>
__device__ __forceinline__ void fx_bias_load(const FxRows<E> &rows, int col, int n, int rot, int lane, float (&b)[MK_FX_HEAD_REGS], float (&bp)[MK_FX_HEAD_REGS]) {
#if MK_HAVE_HYB
  const int half = rot >> 1;
  const float *p = rows.bias;
#pragma unroll
  for (int j = 0; j < MK_FX_HEAD_REGS; j++) b[j] = bp[j] = 0.f;
  if (!p) return;
#pragma unroll
  for (int j = 0; j < MK_FX_HEAD_REGS; j++)
    if (j * 64 < n) {
      const int d = min(j * 64 + lane, n - 1);
      b[j] = p[col + d];
      if (j * 64 < rot) bp[j] = p[col + (d < rot ? (d < half ? d + half : d - half) : d)];
    }
#endif
}
template <typename E>
__device__ __forceinline__ void fx_head_load(CStage &st, const FxRows<E> &rows, int tok, int col, int pos, int lane, FxHead &h) {
  const int D = st.head_dim, rot = (st.flags & MK_F_ROPE) ? st.rot_dims : 0, half = rot >> 1;
  const float *ct = (const float *)st.cos_tab + (size_t)pos * st.ld_cos, *sn = (const float *)st.sin_tab + (size_t)pos * st.ld_cos;
  rows.with_slices([&](auto ns) {
    constexpr int NS = decltype(ns)::value;
#pragma unroll
    for (int j = 0; j < MK_FX_HEAD_REGS; j++)
      if (j * 64 < D) {
        const int d = min(j * 64 + lane, D - 1);
        h.x[j] = rows.template get<NS>(tok, col + d);
        if (j * 64 < rot) {
          const bool in = d < rot, lo = d < half;
          h.xp[j] = rows.template get<NS>(tok, col + (in ? (lo ? d + half : d - half) : d));
          const int ci = in ? (lo ? d : d - half) : 0;
          h.cs[j] = ct[ci];
          h.sn[j] = sn[ci];
        }
      }
  });
#if MK_HAVE_HYB
  fx_bias_load(rows, col, D, rot, lane, h.b, h.bp);
#endif
}
// ... and a value row, which is copied as it is: columns [0, n) of it, lane l holds every 64th
template <typename E>
__device__ __forceinline__ void fx_value_load(const FxRows<E> &rows, int tok, int col, int n, int lane, float (&v)[MK_FX_HEAD_REGS]) {
  rows.with_slices([&](auto ns) {
#pragma unroll
    for (int j = 0; j < MK_FX_HEAD_REGS; j++)
      if (j * 64 < n) v[j] = rows.template get<decltype(ns)::value>(tok, col + min(j * 64 + lane, n - 1));
  });
}
template <typename Put>
__device__ __forceinline__ void fx_head_finish(CStage &st, int lane, FxHead &h, Put put) {
  const int D = st.head_dim, rot = (st.flags & MK_F_ROPE) ? st.rot_dims : 0, half = rot >> 1;
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < MK_FX_HEAD_REGS; j++)
    if (j * 64 < D) {
      const int d = j * 64 + lane;
#if MK_HAVE_HYB
      h.x[j] += h.b[j];
      if (j * 64 < rot) h.xp[j] += h.bp[j];
#endif
      if (j * 64 < rot && d < rot) h.x[j] = d < half ? h.x[j] * h.cs[j] - h.xp[j] * h.sn[j] : h.x[j] * h.cs[j] + h.xp[j] * h.sn[j];
      ss += d < D ? h.x[j] * h.x[j] : 0.f;
    }
  if (st.flags & MK_F_QK_NORM) {
    const float r = 1.f / sqrtf(wave_sum(ss) / (float)D + st.eps);
#pragma unroll
    for (int j = 0; j < MK_FX_HEAD_REGS; j++)
      if (j * 64 < D) h.x[j] *= r;
  }
#if MK_HAVE_DUAL
  if (st.flags & MK_F_ROW_NORM) {
#pragma unroll
    for (int j = 0; j < MK_FX_HEAD_REGS; j++)
      if (j * 64 < D) h.x[j] = (h.x[j] * h.r) * h.w[j];
  }
#endif
#pragma unroll
  for (int j = 0; j < MK_FX_HEAD_REGS; j++)
    if (j * 64 + lane < D) put(j * 64 + lane, h.x[j]);
}

// Cache layout, chosen for the matrix cores (a page is page_size positions of all kv heads):
//   K  [position / 16][kv head][dim / KW][64 lanes][EPC]: lane l holds position l % 16, dims (l / 16) * EPC .. of the KW;
//   V  [position / TP][kv head][dim / 16][64 lanes][EPC]: lane l holds dim l % 16, positions 4 (l / 16) .. + 3 of each
//      16-position sub-tile (sub-tile u in elements 4 u .. 4 u + 3).
// Every operand of a tile is then one contiguous 1 KB request, with no transpose on the way.  Dims are padded with zeros.
template <typename E>
__device__ __forceinline__ size_t fx_k_at(int page, int pp, int ps, int nkv, int g, int nkc, int d) {
  constexpr int EPC = FxType<E>::EPC, KW = FxType<E>::KW;
  return ((((((size_t)page * ps + pp) / 16) * nkv + g) * nkc + d / KW) * 64 + ((d % KW) / EPC) * 16 + (pp & 15)) * EPC + (d % EPC);
}
template <typename E>
__device__ __forceinline__ size_t fx_v_at(int page, int pp, int ps, int nkv, int g, int nvb, int d) {
  constexpr int EPC = FxType<E>::EPC, TP = FxType<E>::TP;
  return ((((((size_t)page * ps + pp) / TP) * nkv + g) * nvb + d / 16) * 64 + ((pp & 15) >> 2) * 16 + (d & 15)) * EPC + ((pp % TP) / 16) * 4 + (pp & 3);
}

// Column the value heads begin at (hybrid kernels: the keys' where a model's values are its keys before rotation).
__device__ __forceinline__ int fx_value_col(CStage &st) {
#if MK_HAVE_HYB
  return st.v_col;
#else
  return (st.num_q_heads + st.num_kv_heads) * st.head_dim;
#endif
}

// Query, key and value rows of an iteration in which some request brings several tokens: a wavefront per (token, head)
// row.  Queries go to the workspace, keys and values to their pages.  (When every request brings one token the attention
// stage does this itself and the stage is skipped.)
template <typename E>
__device__ __forceinline__ void stage_fx_prep(CStage &st, Ctx &c, const MkRuntime &rt, int M) {
  barrier_wait(c);
  constexpr int KW = FxType<E>::KW;
  const FxRows<E> rows = fx_rows<E>(st, c);
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int H = st.num_q_heads, nkv = st.num_kv_heads, D = st.head_dim, DV = st.v_dim;
  const int nkc = (D + KW - 1) / KW, nvb = (DV + 15) / 16, ps = rt.page_size;
  const int per = H + 2 * nkv, total = M * per;
  E *kc = (E *)st.k_cache, *vc = (E *)st.v_cache;
  const int stride = c.G * MK_WAVES;
  auto load = [&](int i, FxHead &h, int &page) {
    const int t = i / per, s = i - t * per;
    const int pos = __builtin_amdgcn_readfirstlane(c.sh_tok[t]);
    page = s < H ? 0 : rt.kv_indices[__builtin_amdgcn_readfirstlane(c.sh_tok[3 * MK_MAX_TOKENS + t]) + pos / ps];
    if (s < H + nkv) {
      fx_head_load<E>(st, rows, t, s * D, pos, lane, h);
#if MK_HAVE_DUAL
      if (st.flags & MK_F_ROW_NORM) {
        const int c0 = s < H ? 0 : H * D, c1 = s < H ? H * D : (H + nkv) * D;
        fx_row_weights(st, s * D, lane, h);
        h.r = 1.f / sqrtf(wave_sum(fx_row_squares<E>((const E *)st.in + (size_t)t * st.ld_in, c0, c1, lane, 64)) / (float)(c1 - c0) + st.eps);
      }
#endif
    } else {
      fx_value_load<E>(rows, t, fx_value_col(st) + (s - H - nkv) * DV, DV, lane, h.x);
#if MK_HAVE_HYB
      fx_bias_load(rows, fx_value_col(st) + (s - H - nkv) * DV, DV, 0, lane, h.b, h.bp);
#endif
    }
  };
  auto finish = [&](int i, FxHead &h, int page) {
    const int t = i / per, s = i - t * per;
    const int pp = __builtin_amdgcn_readfirstlane(c.sh_tok[t]) % ps;
    if (s < H) {
      E *q = (E *)st.q_ws + (size_t)t * st.ld_qws + (size_t)s * nkc * KW;
      fx_head_finish(st, lane, h, [&](int d, float v) { fx_stc(q + d, fx_round<E>(v)); });
      for (int d = D + lane; d < nkc * KW; d += 64) fx_stc(q + d, (E)0);
    } else if (s < H + nkv) {
      fx_head_finish(st, lane, h, [&](int d, float v) { fx_stc(kc + fx_k_at<E>(page, pp, ps, nkv, s - H, nkc, d), fx_round<E>(v)); });
    } else {
      const int g = s - H - nkv;
#if MK_HAVE_HYB
#pragma unroll
      for (int j = 0; j < MK_FX_HEAD_REGS; j++) h.x[j] += h.b[j];
#endif
#pragma unroll
      for (int j = 0; j < MK_FX_HEAD_REGS; j++)
        if (j * 64 + lane < DV) fx_stc(vc + fx_v_at<E>(page, pp, ps, nkv, g, nvb, j * 64 + lane), fx_round<E>(h.x[j]));
    }
  };
  for (int i = c.vid * MK_WAVES + wave; i < total; i += 2 * stride) {
    FxHead h0, h1;
    int p0, p1 = 0;
    load(i, h0, p0);
    if (i + stride < total) load(i + stride, h1, p1);
    finish(i, h0, p0);
    if (i + stride < total) finish(i + stride, h1, p1);
  }
  c.wrote_through = true;
}

// ----------------------------------------------------------------------------- attention
__device__ __forceinline__ f32x4 fx_mma_k(uint16_t, u32x4 a, u32x4 b, f32x4 acc) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), acc, 0, 0, 0);
}
__device__ __forceinline__ f32x4 fx_mma_k(float, u32x4 a, u32x4 b, f32x4 acc) {
#pragma unroll
  for (int j = 0; j < 4; j++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a[j]), __uint_as_float(b[j]), acc, 0, 0, 0);
  return acc;
}
__device__ __forceinline__ float fx_exp2(uint16_t, float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float fx_exp2(float, float x) { return exp2f(x); }

// Work unit = (16 query rows of one request and kv head, slice of VB * 16 value dims, chunk of the cached positions).  A
// query row is a (token, query head of the group) pair, tokens outermost.  The wavefronts of a workgroup take every fourth
// tile of TP positions: scores = K tile x query rows (positions in the rows of the result), so a lane's four results per
// sub-tile are exactly its operand of the product with V (bf16: as value + rounding remainder, which keeps about 16
// mantissa bits of the weights).  Running maximum and sum per query row and wavefront; wavefronts are merged through LDS,
// chunks through the partial buffer by the last workgroup to arrive.  The sink enters once, in the final division.
//
// `single`: every request of the iteration brings one token.  The stage then rotates, normalises and appends the new rows
// itself (the chunk that owns the new position takes its key and value from LDS, nothing of the iteration is read back
// from memory), and the first tiles' rows, which earlier iterations wrote, are requested before the barrier is awaited.
// Otherwise the prep stage has written queries, keys and values.
#define MK_FX_NEG (-1e30f)
// Chunks a unit of NT tiles is split into: none while every wavefront has at most two tiles (a hand-over costs about as
// much), else one tile per wavefront, and two once that would make more than 16 chunks to combine.
__device__ __forceinline__ int fx_chunks(int NT, int cmax) {
  const int rounds = (NT + MK_WAVES - 1) / MK_WAVES;  // tiles of the busiest wavefront without a split
  return rounds <= 2 ? 1 : min(cmax, rounds <= 16 ? rounds : max(16, (rounds + 1) / 2));
}
template <typename E, int KC, int VB>
__device__ __forceinline__ void stage_fx_attn_t(CStage &st, Ctx &c, const MkRuntime &rt, int M, bool single, char *smem) {
  using X = FxType<E>;
  constexpr int EPC = X::EPC, KW = X::KW, TP = X::TP, SUB = X::SUB;
  constexpr int PSTR = VB * 16 + 4, PST = VB * 16 + 32;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int lr = lane & 15, lg = lane >> 4;
  const int nkv = st.num_kv_heads, qpk = st.num_q_heads / nkv, D = st.head_dim, DV = st.v_dim;
  const int nkc = (D + KW - 1) / KW, nkg = (nkc + KC - 1) / KC, nvb = (DV + 15) / 16, nvs = (nvb + VB - 1) / VB;
  const int ps = rt.page_size;
  const u32x4 *kc = (const u32x4 *)st.k_cache, *vc = (const u32x4 *)st.v_cache;
  // LDS
  u32x4 *qs = (u32x4 *)smem;                                   // [nkg * KC][64] query operands
  E *kn = (E *)(smem + nkg * KC * 1024);                       // new key, padded with zeros to nkc * KW
  E *vn = kn + nkc * KW;                                       // new value, padded with zeros to nvb * 16
  float *part = (float *)(smem + (nkg * KC * 1024 + (nkc * KW + nvb * 16) * (int)sizeof(E) + 15) / 16 * 16);  // [4][16][PSTR]
  float *ml = part + MK_WAVES * 16 * PSTR;                     // [4][16] maxima, [4][16] sums
  float *fin = ml + 128;                                       // [4][16] weights, [16] maxima, [16] sums
  float *chk = fin + 96;                                       // [chunks][16] maxima, [chunks][16] sums -> weights
  int *sflag = (int *)(chk + 2 * MK_ATTN_MAX_CHUNKS * 16);
  int *spg = sflag + 4;                                        // page-table entries of the chunk
  // rows of the requests, in row tiles of 16
  int my_n, my_tiles;
  {
    const bool first = lane < M && c.sh_tok[2 * MK_MAX_TOKENS + lane] == lane;
    const unsigned long long fm = __ballot(first), later = lane < 63 ? fm >> (lane + 1) : 0ull;
    my_n = first ? (later ? (int)__ffsll(later) : M - lane) : 0;
    my_tiles = (my_n * qpk + 15) / 16;
  }
  const int tiles_incl = wave_incl_scan(my_tiles, lane);
  const int RT = wave_bcast(tiles_incl, 63);
  const int n_items = RT * nkv * nvs;
  const int cmax = max(1, min(c.G / n_items, MK_ATTN_MAX_CHUNKS));
  const int n_units = n_items * cmax;
  struct Unit {
    int item, cidx, C, g, vs, t0, r0, nrows, p0, p, tb, te, pages, kept, gap;
  };
  // Tiles of a unit are counted without those that none of its rows sees: with a window, `kept` first ones, then `gap` left out.
  const int win = MK_HAVE_HYB ? st.window : 0, keep = MK_HAVE_HYB ? st.keep_first : 0;
  auto phys = [](const Unit &a, int tile) { return MK_HAVE_HYB && tile >= a.kept ? tile + a.gap : tile; };
  auto decode = [&](int u, Unit &a) -> bool {
    a.item = u / cmax;
    a.cidx = u - a.item * cmax;
    a.g = a.item / (RT * nvs);  // kv head outermost: its units sit on adjacent workgroups, i.e. on one die
    const int rem = a.item - a.g * RT * nvs;
    a.vs = rem / RT;
    const int tile = rem - a.vs * RT;
    a.t0 = (int)__ffsll(__ballot(tiles_incl > tile)) - 1;
    const int n = wave_bcast(my_n, a.t0);
    a.r0 = (tile - (wave_bcast(tiles_incl, a.t0) - wave_bcast(my_tiles, a.t0))) * 16;
    a.nrows = min(16, n * qpk - a.r0);
    a.p0 = __builtin_amdgcn_readfirstlane(c.sh_tok[a.t0]);
    a.p = a.p0 + (a.r0 + a.nrows - 1) / qpk;  // newest position any of the rows sees
    int NT = a.p / TP + 1;
    if (MK_HAVE_HYB) {
      const int first = a.p0 + a.r0 / qpk;  // position of the unit's first row
      int oldest = win ? max(0, first - win + 1) : 0;  // oldest position inside its window
#if MK_HAVE_DUAL
      if (st.chunk) oldest = max(oldest, first - first % st.chunk);  // ... and inside its chunk
      a.kept = win || st.chunk ? min((keep + TP - 1) / TP, NT) : NT;
#else
      a.kept = win ? min((keep + TP - 1) / TP, NT) : NT;
#endif
      a.gap = max(0, oldest / TP - a.kept);
      NT -= a.gap;
    }
    a.C = fx_chunks(NT, cmax);
    if (a.cidx >= a.C) return false;
    a.tb = (int)(((long long)NT * a.cidx) / a.C);
    a.te = (int)(((long long)NT * (a.cidx + 1)) / a.C);
    a.pages = __builtin_amdgcn_readfirstlane(c.sh_tok[3 * MK_MAX_TOKENS + a.t0]);
    return true;
  };
  // operands of tile `tile`, dim group kg (page: its page-table entry).  !ok: the same number of loads from one spot.
  auto load_tile = [&](const Unit &a, int tile, int kg, int page, bool ok, u32x4 (&k)[SUB][KC], u32x4 (&v)[VB]) {
    const int pp = (tile * TP) % ps;
    const size_t pt = (size_t)page * ps + pp;
    const u32x4 *kp = kc + (ok ? ((pt / 16) * nkv + a.g) * nkc * 64 : 0) + lane;
    const u32x4 *vp = vc + (ok ? ((pt / TP) * nkv + a.g) * nvb * 64 : 0) + lane;
    const int on = ok ? 64 : 0, su = ok ? nkv * nkc * 64 : 0;
#pragma unroll
    for (int u = 0; u < SUB; u++)
#pragma unroll
      for (int s = 0; s < KC; s++) k[u][s] = kp[u * su + min(kg * KC + s, nkc - 1) * on];
#pragma unroll
    for (int b = 0; b < VB; b++) v[b] = vp[min(a.vs * VB + b, nvb - 1) * on];
  };
  u32x4 kA[SUB][KC], vA[VB], kB[SUB][KC], vB[VB];
  Unit a0;
  const bool have0 = c.vid < n_units && decode(c.vid, a0);
  auto load_first = [&](const Unit &a) {
    const int tile = a.tb + wave;
    const bool ok = tile < a.te;
    const int page = rt.kv_indices[a.pages + phys(a, ok ? tile : a.tb) * TP / ps];
    load_tile(a, phys(a, tile), 0, page, ok, kA, vA);
  };
  const bool early = single && have0 && wave != 0;  // (the polling wavefront keeps its memory queue empty)
  if (early) load_first(a0);
  if (!single && tid == 0) __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");  // the prep stage's rows are read with cached loads
  barrier_wait(c);
  c.wrote_through = true;
  FxRows<E> rows{};
  if (single) rows = fx_rows<E>(st, c);
  const float cap = st.softcap, sc1 = cap > 0.f ? st.sm_scale / cap : st.sm_scale;
  const float LOG2E = 1.4426950408889634f;

  for (int uu = c.vid; uu < n_units; uu += c.G) {
    Unit a;
    const bool first = uu == c.vid;
    int u = uu;
    if (cmax == 1 && ((uu / c.G) & 1)) {  // every other round deals the units in reverse order (contexts differ)
      const int b0 = (uu / c.G) * c.G, bn = min(c.G, n_units - b0);
      u = b0 + bn - 1 - (uu - b0);
    }
    if (first) {
      if (!have0) continue;
      a = a0;
    } else if (!decode(u, a)) {
      continue;
    }
    if (!(first && early)) load_first(a);
    __syncthreads();  // LDS reuse across units
    const int pg_lo = phys(a, a.tb) * TP / ps, npg = min((phys(a, a.te - 1) * TP + TP - 1) / ps, a.p / ps) - pg_lo + 1;
    for (int i = tid; i < npg; i += MK_THREADS) spg[i] = rt.kv_indices[a.pages + pg_lo + i];
    const bool newest = single && a.cidx == a.C - 1;
    // ---- query rows into operand order (and the new key and value)
    if (single) {
#if MK_HAVE_DUAL
      float rq = 0.f, rk = 0.f;
      if (st.flags & MK_F_ROW_NORM) {
        const int nq = st.num_q_heads * D, nk = nkv * D;
        const E *row = (const E *)st.in + (size_t)a.t0 * st.ld_in;
        rq = fx_row_squares<E>(row, 0, nq, tid, MK_THREADS);
        if (newest) rk = fx_row_squares<E>(row, nq, nq + nk, tid, MK_THREADS);
        rq = wave_sum(rq);
        rk = wave_sum(rk);
        if (lane == 0) {
          part[wave] = rq;
          part[4 + wave] = rk;
        }
        __syncthreads();
        rq = 1.f / sqrtf(((part[0] + part[1]) + (part[2] + part[3])) / (float)nq + st.eps);
        rk = 1.f / sqrtf(((part[4] + part[5]) + (part[6] + part[7])) / (float)nk + st.eps);
      }
#endif
      // (everything the row writers below leave out is zeroed: unused query columns, padding dims)
      const u32x4 z = {0u, 0u, 0u, 0u};
      for (int i = tid; i < nkg * KC * 64; i += MK_THREADS)
        if ((i & 15) >= a.nrows || (i >> 6) >= nkc) qs[i] = z;
      E *q = (E *)qs;
      for (int i = tid; i < 16 * (nkc * KW - D); i += MK_THREADS) {
        const int d = D + i / 16;
        if ((i & 15) < a.nrows) q[((d / KW) * 64 + ((d % KW) / EPC) * 16 + (i & 15)) * EPC + d % EPC] = (E)0;
      }
      for (int i = D + tid; i < nkc * KW; i += MK_THREADS) kn[i] = (E)0;
      for (int i = DV + tid; i < nvb * 16; i += MK_THREADS) vn[i] = (E)0;
      // rows 0 .. nrows - 1 are queries, row nrows (the chunk that owns the new position) is the new key; the last
      // wavefront, whose tile has been in flight longest, takes row 0 and with it the first of the second round
      const int n_rows = a.nrows + (newest ? 1 : 0), w_ = MK_WAVES - 1 - wave;
      const bool v_row = newest && w_ == 1;
      const int v_col = fx_value_col(st) + a.g * DV;
      float vv[MK_FX_HEAD_REGS];
      if (v_row) fx_value_load<E>(rows, a.t0, v_col, DV, lane, vv);
#if MK_HAVE_HYB
      float vb[MK_FX_HEAD_REGS], vbp[MK_FX_HEAD_REGS];
      if (v_row) fx_bias_load(rows, v_col, DV, 0, lane, vb, vbp);
#endif
      auto load_row = [&](int r, FxHead &h) {
        fx_head_load<E>(st, rows, a.t0, (r < a.nrows ? a.g * qpk + a.r0 + r : st.num_q_heads + a.g) * D, a.p, lane, h);
#if MK_HAVE_DUAL
        fx_row_weights(st, (r < a.nrows ? a.g * qpk + a.r0 + r : st.num_q_heads + a.g) * D, lane, h);
        h.r = r < a.nrows ? rq : rk;
#endif
      };
      auto put_row = [&](int r, FxHead &h) {
        if (r < a.nrows) fx_head_finish(st, lane, h, [&](int d, float v) { q[((d / KW) * 64 + ((d % KW) / EPC) * 16 + r) * EPC + d % EPC] = fx_round<E>(v); });
        else fx_head_finish(st, lane, h, [&](int d, float v) { kn[d] = fx_round<E>(v); });
      };
      for (int r = w_; r < n_rows; r += 2 * MK_WAVES) {
        FxHead h0, h1;
        load_row(r, h0);
        if (r + MK_WAVES < n_rows) load_row(r + MK_WAVES, h1);
        put_row(r, h0);
        if (r + MK_WAVES < n_rows) put_row(r + MK_WAVES, h1);
      }
      if (v_row) {
#pragma unroll
        for (int j = 0; j < MK_FX_HEAD_REGS; j++)
#if MK_HAVE_HYB
          if (j * 64 + lane < DV) vn[j * 64 + lane] = fx_round<E>(vv[j] + vb[j]);
#else
          if (j * 64 + lane < DV) vn[j * 64 + lane] = fx_round<E>(vv[j]);
#endif
      }
    } else {
      for (int i = tid; i < nkg * KC * 64; i += MK_THREADS) {
        const int s = i >> 6, r = i & 15, R = a.r0 + r;
        u32x4 v = {0u, 0u, 0u, 0u};
        if (r < a.nrows && s < nkc)
          v = ldc_16B((const u32x4 *)((const E *)st.q_ws + (size_t)(a.t0 + R / qpk) * st.ld_qws + (size_t)(a.g * qpk + R % qpk) * nkc * KW + s * KW +
                                      ((i & 63) >> 4) * EPC));
        qs[i] = v;
      }
    }
    __syncthreads();
    if (newest && a.r0 == 0 && a.vs == 0) {  // append the new rows to their page
      const int pp = a.p % ps, page = spg[a.p / ps - pg_lo];
      for (int i = tid; i < nkc * 4; i += MK_THREADS)
        stc_16B((u32x4 *)st.k_cache + (((((size_t)page * ps + pp) / 16) * nkv + a.g) * nkc + (i >> 2)) * 64 + (i & 3) * 16 + (pp & 15), ((const u32x4 *)kn)[i]);
      for (int d = tid; d < DV; d += MK_THREADS) fx_stc((E *)st.v_cache + fx_v_at<E>(page, pp, ps, nkv, a.g, nvb, d), vn[d]);
    }
    // ---- tiles
    const int plim = a.p0 + (a.r0 + min(lr, a.nrows - 1)) / qpk;  // newest position this lane's query row sees
#if MK_HAVE_DUAL
    const int olim = st.chunk ? plim - plim % st.chunk : 0;  // oldest one
    const float sc_row = sc1 * (st.temp ? st.temp[a.g * qpk + (a.r0 + min(lr, a.nrows - 1)) % qpk] : 1.f);
#else
    const float sc_row = sc1;
#endif
    float m = MK_FX_NEG, l = 0.f;
    f32x4 acc[VB], S[SUB];
#pragma unroll
    for (int b = 0; b < VB; b++) acc[b] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int n_mine = a.te - a.tb > wave ? (a.te - a.tb - wave + MK_WAVES - 1) / MK_WAVES : 0;
    auto compute = [&](int tile, int kg, u32x4 (&k)[SUB][KC], u32x4 (&v)[VB]) {
      const bool has_new = single && tile == a.p / TP;
      if (has_new) {
        const u32x4 *kn4 = (const u32x4 *)kn;
#pragma unroll
        for (int u_ = 0; u_ < SUB; u_++)
          if (u_ == (a.p % TP) / 16) {
#pragma unroll
            for (int s = 0; s < KC; s++) {
              const u32x4 x = kn4[min(kg * KC + s, nkc - 1) * 4 + lg];
              if (lr == (a.p & 15)) k[u_][s] = x;
            }
          }
      }
      if (kg == 0) {
#pragma unroll
        for (int u_ = 0; u_ < SUB; u_++) S[u_] = (f32x4){0.f, 0.f, 0.f, 0.f};
      }
#pragma unroll
      for (int s = 0; s < KC; s++) {
        const u32x4 q = qs[(kg * KC + s) * 64 + lane];
#pragma unroll
        for (int u_ = 0; u_ < SUB; u_++) S[u_] = fx_mma_k(E(), k[u_][s], q, S[u_]);
      }
      if (kg + 1 < nkg) return;
      float sc[SUB][4];
      float tm = MK_FX_NEG;
#pragma unroll
      for (int u_ = 0; u_ < SUB; u_++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          float s = S[u_][i] * sc_row;
          if (cap > 0.f) {
            if constexpr (sizeof(E) == 2) {
              const float e = __builtin_amdgcn_exp2f(s * (2.f * LOG2E));
              s = (cap * LOG2E) * (1.f - 2.f * __builtin_amdgcn_rcpf(1.f + e));
            } else {
              s = (cap * LOG2E) * tanhf(s);
            }
          } else {
            s *= LOG2E;
          }
          const int at = tile * TP + u_ * 16 + lg * 4 + i;
          bool seen = at <= plim;
          if (MK_HAVE_HYB) seen = seen && (win == 0 || plim - at < win || at < keep);
#if MK_HAVE_DUAL
          seen = seen && at >= olim;
#endif
          s = seen ? s : MK_FX_NEG;
          sc[u_][i] = s;
          tm = fmaxf(tm, s);
        }
      tm = groups_max(tm);
      if (__any(tm > m)) {
        const float nm = fmaxf(m, tm), corr = fx_exp2(E(), m - nm);
        m = nm;
        l *= corr;
#pragma unroll
        for (int b = 0; b < VB; b++) acc[b] *= corr;
      }
#pragma unroll
      for (int u_ = 0; u_ < SUB; u_++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          sc[u_][i] = sc[u_][i] > 0.5f * MK_FX_NEG ? fx_exp2(E(), sc[u_][i] - m) : 0.f;
          l += sc[u_][i];
        }
      if (has_new) {
#pragma unroll
        for (int b = 0; b < VB; b++) {
          const E x = vn[min(a.vs * VB + b, nvb - 1) * 16 + lr];
          const int slot = ((a.p % TP) / 16) * 4 + (a.p & 3);
#pragma unroll
          for (int w = 0; w < 4; w++) {
            uint32_t nv;
            bool here;
            if constexpr (sizeof(E) == 2) {
              here = w == (slot >> 1);
              nv = (slot & 1) ? (v[b][w] & 0xffffu) | ((uint32_t)x << 16) : (v[b][w] & 0xffff0000u) | (uint32_t)x;
            } else {
              here = w == slot;
              nv = __float_as_uint(x);
            }
            if (here && lg == ((a.p & 15) >> 2)) v[b][w] = nv;
          }
        }
      }
      if ((tile + 1) * TP - 1 > a.p) {  // values behind the newest position belong to nobody: whatever they are, 0 x them is 0
#pragma unroll
        for (int b = 0; b < VB; b++)
#pragma unroll
          for (int w = 0; w < 4; w++) {
            if constexpr (sizeof(E) == 2) {
              const int q = tile * TP + (w >> 1) * 16 + lg * 4 + (w & 1) * 2;
              v[b][w] = q > a.p ? 0u : (q + 1 > a.p ? v[b][w] & 0xffffu : v[b][w]);
            } else {
              if (tile * TP + lg * 4 + w > a.p) v[b][w] = 0u;
            }
          }
      }
      if constexpr (sizeof(E) == 2) {
        u32x4 hi, lo;
#pragma unroll
        for (int w = 0; w < 4; w++) {
          const float x0 = sc[w >> 1][(w & 1) * 2], x1 = sc[w >> 1][(w & 1) * 2 + 1];
          hi[w] = pack2(x0, x1);
          lo[w] = pack2(x0 - bf_lo(hi[w]), x1 - bf_hi(hi[w]));
        }
#pragma unroll
        for (int b = 0; b < VB; b++) {
          acc[b] = fx_mma_k(E(), v[b], hi, acc[b]);
          acc[b] = fx_mma_k(E(), v[b], lo, acc[b]);
        }
      } else {
        u32x4 pw;
#pragma unroll
        for (int w = 0; w < 4; w++) pw[w] = __float_as_uint(sc[0][w]);
#pragma unroll
        for (int b = 0; b < VB; b++) acc[b] = fx_mma_k(E(), v[b], pw, acc[b]);
      }
    };
    const int n_it = n_mine * nkg;
    int tile = a.tb + wave, kg = 0;
    auto next = [&](int &tl, int &kk) {
      if (++kk == nkg) {
        kk = 0;
        tl += MK_WAVES;
      }
    };
    for (int it = 0; it < n_it; it += 2) {
      int tl = tile, kk = kg;
      next(tl, kk);
      bool ok = it + 1 < n_it;
      load_tile(a, phys(a, tl), kk, ok ? spg[phys(a, tl) * TP / ps - pg_lo] : 0, ok, kB, vB);
      compute(phys(a, tile), kg, kA, vA);
      if (!ok) break;
      tile = tl;
      kg = kk;
      next(tl, kk);
      ok = it + 2 < n_it;
      load_tile(a, phys(a, tl), kk, ok ? spg[phys(a, tl) * TP / ps - pg_lo] : 0, ok, kA, vA);
      compute(phys(a, tile), kg, kB, vB);
      tile = tl;
      kg = kk;
    }
    // ---- wavefronts of the workgroup
    l = groups_sum(l);
#pragma unroll
    for (int b = 0; b < VB; b++) *(f32x4 *)(part + (wave * 16 + lr) * PSTR + b * 16 + lg * 4) = acc[b];
    if (lg == 0) {
      ml[wave * 16 + lr] = m;
      ml[64 + wave * 16 + lr] = l;
    }
    __syncthreads();
    const float *sink = (const float *)st.sink;
    auto sink_of = [&](int r) -> float { return sink ? sink[a.g * qpk + (a.r0 + min(r, a.nrows - 1)) % qpk] * LOG2E : -INFINITY; };
    if (tid < 16) {
      float M_ = MK_FX_NEG, L_ = 0.f;
#pragma unroll
      for (int w = 0; w < MK_WAVES; w++) M_ = fmaxf(M_, ml[w * 16 + tid]);
#pragma unroll
      for (int w = 0; w < MK_WAVES; w++) {
        const float e = exp2f(ml[w * 16 + tid] - M_);
        fin[w * 16 + tid] = e;
        L_ += ml[64 + w * 16 + tid] * e;
      }
      if (a.C == 1) {
        const float inv = 1.f / (L_ + exp2f(sink_of(tid) - M_));
#pragma unroll
        for (int w = 0; w < MK_WAVES; w++) fin[w * 16 + tid] *= inv;
      } else {
        float *pb = (float *)rt.attn_part + ((size_t)u * 16 + tid) * PST + VB * 16;
        stc_f32(pb, M_);
        stc_f32(pb + 1, L_);
      }
    }
    __syncthreads();
    const int dv0 = a.vs * VB * 16;
    auto emit = [&](int r, int d, const f32x4 &o) {
      const int R = a.r0 + r;
      E *row = (E *)st.out + (size_t)(a.t0 + R / qpk) * st.ld_out + (size_t)(a.g * qpk + R % qpk) * DV;
      const float q[4] = {o[0], o[1], o[2], o[3]};
      fx_stc4(row, dv0 + d, DV, q);
    };
    for (int i = tid; i < 16 * VB * 4; i += MK_THREADS) {
      const int r = i / (VB * 4), d = (i - r * (VB * 4)) * 4;
      if (r >= a.nrows || dv0 + d >= DV) continue;
      f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int w = 0; w < MK_WAVES; w++) o += *(const f32x4 *)(part + (w * 16 + r) * PSTR + d) * fin[w * 16 + r];
      if (a.C == 1) emit(r, d, o);
      else stc_16B((u32x4 *)((float *)rt.attn_part + ((size_t)u * 16 + r) * PST + d), __builtin_bit_cast(u32x4, o));
    }
    if (a.C == 1) continue;
    // ---- chunks: the last workgroup to arrive combines them
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (tid == 0) {
      unsigned *cnt = rt.attn_cnt + (size_t)a.item * 32;
      const int last = __hip_atomic_fetch_add(cnt, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (unsigned)(a.C - 1);
      if (last) __hip_atomic_store(cnt, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      *sflag = last;
    }
    __syncthreads();
    if (!*sflag) continue;
    const float *pb = (const float *)rt.attn_part + (size_t)a.item * cmax * 16 * PST;
    for (int i = tid; i < a.C * 16; i += MK_THREADS) {
      chk[i] = ldc_f32(pb + (size_t)i * PST + VB * 16);
      chk[MK_ATTN_MAX_CHUNKS * 16 + i] = ldc_f32(pb + (size_t)i * PST + VB * 16 + 1);
    }
    __syncthreads();
    if (tid < 16) {
      float M_ = MK_FX_NEG, L_ = 0.f;
      for (int q = 0; q < a.C; q++) M_ = fmaxf(M_, chk[q * 16 + tid]);
      for (int q = 0; q < a.C; q++) {
        const float e = exp2f(chk[q * 16 + tid] - M_);
        L_ += chk[MK_ATTN_MAX_CHUNKS * 16 + q * 16 + tid] * e;
        chk[q * 16 + tid] = e;
      }
      fin[tid] = 1.f / (L_ + exp2f(sink_of(tid) - M_));
    }
    __syncthreads();
    for (int i = tid; i < 16 * VB * 4; i += MK_THREADS) {
      const int r = i / (VB * 4), d = (i - r * (VB * 4)) * 4;
      if (r >= a.nrows || dv0 + d >= DV) continue;
      f32x4 o = {0.f, 0.f, 0.f, 0.f};
      for (int q0 = 0; q0 < a.C; q0 += 8) {
        f32x4 x[8];
#pragma unroll
        for (int q = 0; q < 8; q++) x[q] = fx_ldc_quad(pb + ((size_t)min(q0 + q, a.C - 1) * 16 + r) * PST + d);
#pragma unroll
        for (int q = 0; q < 8; q++)
          if (q0 + q < a.C) o += x[q] * chk[(q0 + q) * 16 + r];
      }
      emit(r, d, o * fin[r]);
    }
  }
}
template <typename E>
__device__ __forceinline__ void stage_fx_attn(CStage &st, Ctx &c, const MkRuntime &rt, int M, bool single, char *smem) {
  if constexpr (sizeof(E) == 2) {
    if (st.v_tiles == 4) {
      if (st.k_tiles == 2) stage_fx_attn_t<E, 2, 4>(st, c, rt, M, single, smem);
      else stage_fx_attn_t<E, 4, 4>(st, c, rt, M, single, smem);
    } else {
      stage_fx_attn_t<E, 4, 8>(st, c, rt, M, single, smem);
    }
  } else {
    stage_fx_attn_t<E, 8, 8>(st, c, rt, M, single, smem);
  }
}

// ----------------------------------------------------------------------------- 32-bit linear
// out[m, n] = sum_k x[m, k] W[n, k] in true 32-bit (v_mfma_f32_16x16x4_f32), optional SwiGLU epilogue.  A workgroup owns a
// range of 16-column output tiles and all rows; its wavefronts split K and are reduced through LDS in a fixed order.
__device__ __forceinline__ float fx_glu_f32(CStage &st, float g, float u) {
#if MK_HAVE_DUAL
  if (st.flags & MK_F_GELU) return 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g))) * u;
#endif
  return g / (1.f + expf(-g)) * u;
}
template <int MT>
__device__ __forceinline__ void stage_fx_linear_f32(CStage &st, Ctx &c, int M, char *smem) {
  if (threadIdx.x == 0) __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
  barrier_wait(c);
  c.wrote_through = true;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int lr = lane & 15, lg = lane >> 4;
  const bool silu = st.flags & MK_F_SILU;
  const int K = st.k, n_out = silu ? st.n / 2 : st.n, half = st.silu_half;
  const int ntiles = (n_out + 15) / 16;
  const int t_begin = (int)(((long long)c.vid * ntiles) / c.G), t_end = (int)(((long long)(c.vid + 1) * ntiles) / c.G);
  const int kq = ((K / 16 + MK_WAVES - 1) / MK_WAVES) * 16;
  const int kbeg = min(K, wave * kq), kend = min(K, kbeg + kq);
  f32x4 *red = (f32x4 *)smem;  // [waves][2][MT][64]
  const float *xrow[MT];
#pragma unroll
  for (int mt = 0; mt < MT; mt++) xrow[mt] = (const float *)st.in + (size_t)min(mt * 16 + lr, M - 1) * st.ld_in + lg * 4;
  for (int ot = t_begin; ot < t_end; ot++) {
    const int o = min(ot * 16 + lr, n_out - 1);
    int vr = o;
    if (silu) vr = (o / half) * 2 * half + (o % half);
    const float *w0 = (const float *)weight_row(st.w, vr, K / 4) + lg * 4;
    const float *w1 = silu ? (const float *)weight_row(st.w, vr + half, K / 4) + lg * 4 : w0;
    f32x4 acc[2][MT];
#pragma unroll
    for (int mt = 0; mt < MT; mt++) acc[0][mt] = acc[1][mt] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int k = kbeg; k < kend; k += 16) {
      const f32x4 a0 = *(const f32x4 *)(w0 + k), a1 = *(const f32x4 *)(w1 + k);
      f32x4 b[MT];
#pragma unroll
      for (int mt = 0; mt < MT; mt++) b[mt] = *(const f32x4 *)(xrow[mt] + k);
#pragma unroll
      for (int j = 0; j < 4; j++)
#pragma unroll
        for (int mt = 0; mt < MT; mt++) {
          acc[0][mt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a0[j], b[mt][j], acc[0][mt], 0, 0, 0);
          if (silu) acc[1][mt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a1[j], b[mt][j], acc[1][mt], 0, 0, 0);
        }
    }
    __syncthreads();
#pragma unroll
    for (int h = 0; h < 2; h++)
#pragma unroll
      for (int mt = 0; mt < MT; mt++) red[((wave * 2 + h) * MT + mt) * 64 + lane] = acc[h][mt];
    __syncthreads();
    for (int e = tid; e < MT * 64; e += MK_THREADS) {
      const int l = e & 63, mt = e >> 6, m = mt * 16 + (l & 15);
      f32x4 v = red[mt * 64 + l], g = red[(MT + mt) * 64 + l];
#pragma unroll
      for (int w = 1; w < MK_WAVES; w++) {
        v += red[((w * 2) * MT + mt) * 64 + l];
        g += red[((w * 2 + 1) * MT + mt) * 64 + l];
      }
      if (m < M) {
        float r[4];
#pragma unroll
        for (int i = 0; i < 4; i++) r[i] = silu ? fx_glu_f32(st, v[i], g[i]) : linear_act(st, v[i]);
        fx_stc4((float *)st.out + (size_t)m * st.ld_out, ot * 16 + (l >> 4) * 4, n_out, r);
      }
    }
  }
}

// Greedy sampling over 32-bit logits, stage 1 (stage 2 is stage_argmax_reduce): one wavefront per token.
__device__ __forceinline__ void stage_fx_argmax_f32(CStage &st, Ctx &c, const MkRuntime &rt, int M) {
  barrier_wait(c);
  const int n = st.n, per = (n + c.G - 1) / c.G, c0 = c.vid * per, c1 = min(n, c0 + per);
  float *pv = rt.argmax_pv ? rt.argmax_pv : (float *)st.aux0;
  int *pi = rt.argmax_pv ? rt.argmax_pi : (int *)st.aux1;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  for (int t = wave; t < M; t += MK_WAVES) {
    const float *row = (const float *)st.in + (size_t)t * st.ld_in;
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int i = c0 + lane; i < c1; i += 64) {
      const float v = ldc_f32(row + i);
      if (v > best) {
        best = v;
        bi = i;
      }
    }
    wave_argmax(best, bi);
    if (lane == 0) {
      pv[t * c.G + c.vid] = best;
      pi[t * c.G + c.vid] = bi;
    }
  }
}
