// Latent attention, the generalised delta rule and what goes with them (part of the persistent kernel, included by
// mk_kernel.hip behind mk_flex.hip, whose conventions it keeps: sizes and constants are descriptor fields, E is the type of
// activations, weights and cached rows, everything named in 32 bits is 32-bit in both builds).
//   * stage_mx_prenorm        residual sum (the summand optionally RMS-normalised first), then an RMS norm in equal parts;
//   * stage_mx_latent_prep    query latents and key latents normalised, shared key part rotated, row appended to its page;
//   * stage_mx_head_linear    one small matrix per head, operands in matrix-core order; optional gelu * table-row epilogue;
//   * stage_mx_latent_attn /  attention over cached latents, which are keys and values of all heads at once;
//     stage_mx_latent_merge
//   * stage_mx_delta          recurrence S' = diag(w) S - (a u)(u^T S) + k v^T, o = S'^T r with its gates, norm and state;
//   * mx_glu                  clamped gated activation, run by workgroups beside the latent_prep and delta stages.

// Index that deals consecutive work over the dies first (a handful of units then spreads over all of them).
__device__ __forceinline__ int mx_spread(const Ctx &c) { return c.even_xcds ? c.rank * c.nxcd + c.xi : c.vid; }

// Index of a wavefront among those of the grid, the wavefronts that do not poll the barrier first.
__device__ __forceinline__ int mx_wave_item(const Ctx &c, int wave) { return mx_spread(c) + (MK_WAVES - 1 - wave) * c.G; }

// 1 / (1 + exp(-z)) and tanh(z): hardware exp2 and reciprocal next to 16-bit operands, library functions in the 32-bit build
__device__ __forceinline__ float mx_sigmoid(uint16_t, float z) { return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }
__device__ __forceinline__ float mx_sigmoid(float, float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float mx_tanh(uint16_t, float z) { return 1.f - 2.f * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(2.8853900817779268f * z)); }
__device__ __forceinline__ float mx_tanh(float, float z) { return tanhf(z); }

// A quad of 32-bit values written through to memory in one store (the same visibility as stc_f32).
__device__ __forceinline__ void mx_stc_quad(float *p, f32x4 v) {
  asm volatile("global_store_dwordx4 %0, %1, off sc1" ::"v"((const MK_GLOBAL void *)(unsigned long long)p), "v"(v) : "memory");
}

// Values of a norm stage's summand: this thread's NS quads of row `y`, at(j) the index of quad j.  Hybrid kernels: with `places` the sum of
// st.slots rows of the token, st.ld_slot apart, weighted by `w`; the quads of SQ rows are requested at once.  (A bias is added by the caller, who has
// it in advance.)
template <typename E, int NS, typename At>
__device__ __forceinline__ void mx_summands(CStage &st, const E *y, const float *w, bool places, f32x4 (&v)[NS], At at) {
#if MK_HAVE_HYB
  if (places) {
    constexpr int SQ = NS <= 4 ? 4 : 1;
#pragma unroll
    for (int j = 0; j < NS; j++) v[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int q0 = 0; q0 < st.slots; q0 += SQ) {
      f32x4 x[SQ][NS];
      float f[SQ];
#pragma unroll
      for (int q = 0; q < SQ; q++) {
        const int r = min(q0 + q, st.slots - 1);
        f[q] = q0 + q < st.slots ? ldc_f32(w + r) : 0.f;
#pragma unroll
        for (int j = 0; j < NS; j++) x[q][j] = fx_ldc_quad(y + (size_t)r * st.ld_slot + 4 * at(j));
      }
#pragma unroll
      for (int q = 0; q < SQ; q++)
#pragma unroll
        for (int j = 0; j < NS; j++) v[j] += x[q][j] * f[q];
    }
    return;
  }
#endif
#pragma unroll
  for (int j = 0; j < NS; j++) v[j] = fx_ldc_quad(y + 4 * at(j));
}
// ... one quad
template <typename E>
__device__ __forceinline__ f32x4 mx_summand(CStage &st, const E *y, const float *w, int s) {
  f32x4 v[1];
  mx_summands<E, 1>(st, y, w, MK_HAVE_HYB && st.slots, v, [&](int) { return s; });
  return v[0];
}

#if MK_HAVE_DUAL
// Convolution over time of normed rows, added to them (see mk_dual.hip): one quad of a row whose request brings this one token.  h:
// the row's values as they are stored, ring: the request's ring of st.taps rows.  Taps b0 .. (counted back from the token's own).
template <typename E>
__device__ __forceinline__ f32x4 mx_ring_conv(CStage &st, const E *ring, int n, int pos, int q, int b0, f32x4 acc) {
  const int taps = st.taps;
  for (int b = b0; b < taps; b += 4) {
    f32x4 v[4], g[4];
#pragma unroll
    for (int y = 0; y < 4; y++) {
      const int back = min(b + y, taps - 1);
      v[y] = fx_ldc_quad(ring + (size_t)(max(pos - back, 0) % taps) * n + 4 * q);
      g[y] = fx_ld_quad((const E *)st.conv_w + (size_t)(taps - 1 - back) * n + 4 * q);
    }
#pragma unroll
    for (int y = 0; y < 4; y++)
#pragma unroll
      for (int e = 0; e < 4; e++) acc[e] = b + y < taps && b + y <= pos ? fmaf(v[y][e], g[y][e], acc[e]) : acc[e];
  }
  return acc;
}
#endif

// ----------------------------------------------------------------------------- residual sum + norm in parts
// v = x + alpha * f(y),  f(y) = y or y / sqrt(mean(y^2) + norm_eps) * y_norm_w;  out2 = v (32-bit);  out = the RMS norm of v in
// st.norm_groups equal parts times norm_w (norm_groups 0: v itself), rounded to E.  Rows are st.n long, st.k of them real (the
// rest is zero in every operand).  A workgroup per row.
// Dual kernels: v = x + alpha * y_scale f(y) + y2_scale y2 (both factors element by element; `slots` then belongs to y2), and when every
// request brings one token also out3 = the normed row plus its convolution over time, which keeps the row in the request's ring.
template <typename E, int NS>
__device__ __forceinline__ void stage_mx_prenorm_t(CStage &st, Ctx &c, int M, bool single, char *smem) {
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), n4 = st.n / 4;
  float *red = (float *)smem, *gs = red + 64, *row = gs + MK_MX_MAX_GROUPS;
  const int ng = st.norm_groups, gl = ng ? st.k / ng : st.k;
  const f32x4 *w4 = (const f32x4 *)st.norm_w, *yw4 = (const f32x4 *)st.y_norm_w;
  const float *xr = (const float *)st.res;
  const int t0 = mx_spread(c);
  f32x4 g[NS], x[NS];
  auto at = [&](int j) { return min(tid + j * MK_THREADS, n4 - 1); };
  auto load_x = [&](int t) {
#pragma unroll
    for (int j = 0; j < NS; j++) x[j] = fx_ldc_quad(xr + (size_t)t * st.ld_res + 4 * at(j));
  };
  if (ng) {
#pragma unroll
    for (int j = 0; j < NS; j++) g[j] = w4[at(j)];
  }
#if MK_HAVE_HYB  // (weights are requested before the barrier is awaited)
  f32x4 yw[NS], yb[NS];
  const f32x4 *yb4 = (const f32x4 *)st.in_bias;
  if (yw4) {
#pragma unroll
    for (int j = 0; j < NS; j++) yw[j] = yw4[at(j)];
  }
  if (yb4) {
#pragma unroll
    for (int j = 0; j < NS; j++) yb[j] = yb4[at(j)];
  }
#endif
#if MK_HAVE_DUAL
  // factors and the convolution's weights (short rows: in advance; long ones: where they are used)
  constexpr bool AHEAD = NS <= 4;
  constexpr int NA = AHEAD ? NS : 1, TA = AHEAD ? 4 : 1;
  const f32x4 one = {1.f, 1.f, 1.f, 1.f};
  f32x4 ys[NA], y2s[NA], cw[NA][TA], rg[NA][TA];
  if constexpr (AHEAD) {
#pragma unroll
    for (int j = 0; j < NS; j++) {
      ys[j] = st.y_scale ? ((const f32x4 *)st.y_scale)[at(j)] : one;
      y2s[j] = st.y2_scale ? ((const f32x4 *)st.y2_scale)[at(j)] : one;
    }
    if (st.conv_w && single) {
#pragma unroll
      for (int b = 0; b < TA; b++)
#pragma unroll
        for (int j = 0; j < NS; j++) cw[j][b] = fx_ld_quad((const E *)st.conv_w + (size_t)(st.taps - 1 - min(b, st.taps - 1)) * st.n + 4 * at(j));
    }
  }
  auto ys_at = [&](int j) { return AHEAD ? ys[AHEAD ? j : 0] : st.y_scale ? ((const f32x4 *)st.y_scale)[at(j)] : one; };
  auto y2s_at = [&](int j) { return AHEAD ? y2s[AHEAD ? j : 0] : st.y2_scale ? ((const f32x4 *)st.y2_scale)[at(j)] : one; };
#endif
  // the residual row was written at least one barrier earlier than y: requested before the barrier is awaited (not by the
  // wavefront that polls it)
#if MK_HAVE_HYB
  auto yw_at = [&](int j) { return yw[j]; };
#else
  auto yw_at = [&](int j) { return yw4[at(j)]; };
#endif
  const bool pre = (st.flags & MK_F_RES_EARLY) && t0 < M && tid >= 64;
  if (pre) load_x(t0);
  barrier_wait(c);
  for (int t = t0; t < M; t += c.G) {
    if (!(pre && t == t0)) load_x(t);
#if MK_HAVE_DUAL
    const bool conv = st.conv_w && single;
    const int pos = __builtin_amdgcn_readfirstlane(c.sh_tok[t]), taps = st.taps;
    E *ring = conv ? (E *)st.tail + (size_t)__builtin_amdgcn_readfirstlane(c.state_ids[__builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + t])]) * taps * st.n : nullptr;
    if constexpr (AHEAD) {
      if (conv) {
#pragma unroll
        for (int b = 1; b < TA; b++)
#pragma unroll
          for (int j = 0; j < NS; j++) rg[j][b] = fx_ldc_quad(ring + (size_t)(max(pos - min(b, taps - 1), 0) % taps) * st.n + 4 * at(j));
      }
    }
#endif
    if (st.in) {
      f32x4 y[NS];
      const float *sw = MK_HAVE_HYB ? st.slot_w + (size_t)t * st.ld_slot_w : nullptr;
#if MK_HAVE_DUAL
      mx_summands<E, NS>(st, (const E *)st.in + (size_t)t * st.ld_in, sw, st.slots && !st.y2, y, at);
      if (st.y2) {
        f32x4 y2[NS];
        mx_summands<E, NS>(st, (const E *)st.y2 + (size_t)t * st.ld_y2, sw, st.slots, y2, at);
#pragma unroll
        for (int j = 0; j < NS; j++) {
          const f32x4 f2 = y2s_at(j);
#pragma unroll
          for (int e = 0; e < 4; e++) x[j][e] = fmaf(f2[e], y2[j][e], x[j][e]);
        }
      }
#else
      mx_summands<E, NS>(st, (const E *)st.in + (size_t)t * st.ld_in, sw, MK_HAVE_HYB && st.slots, y, at);
#endif
      float f = st.alpha;
#if MK_HAVE_HYB
      if (yb4) {
#pragma unroll
        for (int j = 0; j < NS; j++) y[j] += yb[j];
      }
#endif
      if (yw4) {
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < NS; j++)
          if (tid + j * MK_THREADS < n4) ss += y[j][0] * y[j][0] + y[j][1] * y[j][1] + y[j][2] * y[j][2] + y[j][3] * y[j][3];
        ss = block_sum(ss, red);
        const float r = 1.f / sqrtf(ss / (float)st.k + st.norm_eps);
#pragma unroll
        for (int j = 0; j < NS; j++) y[j] = (y[j] * r) * yw_at(j);
      }
#if MK_HAVE_DUAL
      if (st.y_scale) {
#pragma unroll
        for (int j = 0; j < NS; j++) y[j] *= ys_at(j);
      }
#endif
#pragma unroll
      for (int j = 0; j < NS; j++)
#pragma unroll
        for (int e = 0; e < 4; e++) x[j][e] = fmaf(f, y[j][e], x[j][e]);
    }
    if (ng > 1) {
#pragma unroll
      for (int j = 0; j < NS; j++)
        if (tid + j * MK_THREADS < n4) *(f32x4 *)(row + 4 * (tid + j * MK_THREADS)) = x[j];
      __syncthreads();
      for (int q = wave; q < ng; q += MK_WAVES) {
        float ss = 0.f;
        for (int i = lane; i < gl; i += 64) ss += row[q * gl + i] * row[q * gl + i];
        ss = wave_sum(ss);
        if (lane == 0) gs[q] = 1.f / sqrtf(ss / (float)gl + st.eps);
      }
      __syncthreads();
    } else if (ng == 1) {
      float ss = 0.f;
#pragma unroll
      for (int j = 0; j < NS; j++)
        if (tid + j * MK_THREADS < n4) ss += x[j][0] * x[j][0] + x[j][1] * x[j][1] + x[j][2] * x[j][2] + x[j][3] * x[j][3];
      ss = block_sum(ss, red + 16);
      if (tid == 0) gs[0] = 1.f / sqrtf(ss / (float)gl + st.eps);
      __syncthreads();
    }
#pragma unroll
    for (int j = 0; j < NS; j++)
      if (tid + j * MK_THREADS < n4) {
        const int s = tid + j * MK_THREADS;
        if (st.out2) fx_stc_quad((float *)st.out2 + (size_t)t * st.ld_out2 + 4 * s, x[j]);
        f32x4 o = x[j];
        if (ng) {
          const int q0 = min(4 * s / gl, ng - 1), q3 = min((4 * s + 3) / gl, ng - 1);
#pragma unroll
          for (int e = 0; e < 4; e++) o[e] = (o[e] * gs[q0 == q3 ? q0 : min((4 * s + e) / gl, ng - 1)]) * g[j][e];
        }
        if (st.out) fx_stc_quad((E *)st.out + (size_t)t * st.ld_out + 4 * s, o);
#if MK_HAVE_DUAL
        if (conv) {
          f32x4 h, acc;
#pragma unroll
          for (int e = 0; e < 4; e++) h[e] = fx_val(fx_round<E>(o[e]));
          acc = h;
          if constexpr (AHEAD) {
#pragma unroll
            for (int b = 0; b < TA; b++)
#pragma unroll
              for (int e = 0; e < 4; e++) acc[e] = b < taps && b <= pos ? fmaf(b ? rg[j][b][e] : h[e], cw[j][b][e], acc[e]) : acc[e];
            if (taps > TA) acc = mx_ring_conv<E>(st, ring, st.n, pos, s, TA, acc);
          } else {
            const f32x4 w0 = fx_ld_quad((const E *)st.conv_w + (size_t)(taps - 1) * st.n + 4 * s);
#pragma unroll
            for (int e = 0; e < 4; e++) acc[e] = fmaf(w0[e], h[e], acc[e]);
            acc = mx_ring_conv<E>(st, ring, st.n, pos, s, 1, acc);
          }
          fx_stc_quad((E *)st.out3 + (size_t)t * st.ld_out3 + 4 * s, acc);
          fx_stc_quad(ring + (size_t)(pos % taps) * st.n + 4 * s, h);
        }
#endif
      }
    __syncthreads();
  }
  c.wrote_through = true;
}
#if MK_HAVE_DUAL
template <typename E, typename Put>
__device__ __forceinline__ void mx_norm_row(const E *src, const float *w, int n, float eps, int lane, Put put);
// Rows that are only normalised, in parts of whole quads: a wavefront per (row, part).
template <typename E>
__device__ __forceinline__ void stage_mx_norm_parts(CStage &st, Ctx &c, int M) {
  barrier_wait(c);
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), ng = st.norm_groups, gl = st.k / ng;
  for (int i = mx_wave_item(c, wave); i < M * ng; i += c.G * MK_WAVES) {
    const int t = i / ng, q = i - t * ng;
    E *o = (E *)st.out + (size_t)t * st.ld_out + q * gl;
    mx_norm_row<float>((const float *)st.res + (size_t)t * st.ld_res + q * gl, (const float *)st.norm_w + q * gl, gl, st.eps, lane, [&](int s, f32x4 v) { fx_stc_quad(o + 4 * s, v); });
  }
  c.wrote_through = true;
}
#endif
template <typename E>
__device__ __forceinline__ void stage_mx_prenorm(CStage &st, Ctx &c, int M, bool single, char *smem) {
#if MK_HAVE_DUAL
  if (!st.in && !st.out2 && st.out && !st.conv_w && st.norm_groups && (st.k / st.norm_groups) % 4 == 0 && st.k / st.norm_groups <= MK_MX_MAX_NORM_ROW) {
    stage_mx_norm_parts<E>(st, c, M);
    return;
  }
#endif
  if (st.n <= 4 * 4 * MK_THREADS) stage_mx_prenorm_t<E, 4>(st, c, M, single, smem);
  else stage_mx_prenorm_t<E, 12>(st, c, M, single, smem);
}

// The same in front of a single-token bf16 linear, whose input row it leaves in LDS (virtual workgroup 0 also stores the rows).
__device__ __forceinline__ void mx_x_m1_prenorm(CStage &st, const Ctx &c, uint32_t *xs, float *red) {
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), k4 = st.k / 4, ng = st.norm_groups, gl = st.k_real / ng;
  f32x4 *vs = (f32x4 *)((char *)xs + MK_MOE_OFFSET);  // the sum, 32-bit
  float *gs = (float *)((char *)xs + MK_MOE_OFFSET + 12 * 4 * 4 * MK_THREADS);
  float f = 1.f;
  if (st.y_in && st.y_norm_w) {
    float ss = 0.f;
    for (int i = tid; i < k4; i += MK_THREADS) {
      f32x4 y = mx_summand<uint16_t>(st, (const uint16_t *)st.y_in, MK_HAVE_HYB ? st.slot_w : nullptr, i);
      if (MK_HAVE_HYB && st.in_bias) y += ((const f32x4 *)st.in_bias)[i];
      ss += y[0] * y[0] + y[1] * y[1] + y[2] * y[2] + y[3] * y[3];
    }
    f = 1.f / sqrtf(block_sum(ss, red) / (float)st.k_real + st.norm_eps);
  }
  for (int i = tid; i < k4; i += MK_THREADS) {
    f32x4 v = fx_ldc_quad((const float *)st.res + 4 * i);
    if (st.y_in) {
      f32x4 y = mx_summand<uint16_t>(st, (const uint16_t *)st.y_in, MK_HAVE_HYB ? st.slot_w : nullptr, i);
      if (MK_HAVE_HYB && st.in_bias) y += ((const f32x4 *)st.in_bias)[i];
      if (st.y_norm_w) y = (y * f) * ((const f32x4 *)st.y_norm_w)[i];
#pragma unroll
      for (int e = 0; e < 4; e++) v[e] = fmaf(st.alpha, y[e], v[e]);
    }
    vs[i] = v;
    if (c.vid == 0 && st.out2) stc_16B((u32x4 *)st.out2 + i, __builtin_bit_cast(u32x4, v));
  }
  __syncthreads();
  for (int q = wave; q < ng; q += MK_WAVES) {
    float ss = 0.f;
    for (int i = lane; i < gl; i += 64) ss += ((const float *)vs)[q * gl + i] * ((const float *)vs)[q * gl + i];
    ss = wave_sum(ss);
    if (lane == 0) gs[q] = 1.f / sqrtf(ss / (float)gl + st.eps);
  }
  __syncthreads();
  for (int i = tid; i < k4; i += MK_THREADS) {
    const f32x4 g = ((const f32x4 *)st.norm_w)[i], v = vs[i];
    f32x4 o;
#pragma unroll
    for (int e = 0; e < 4; e++) o[e] = (v[e] * gs[min((4 * i + e) / gl, ng - 1)]) * g[e];
    const unsigned long long h = (unsigned long long)pack2(o[0], o[1]) | ((unsigned long long)pack2(o[2], o[3]) << 32);
    ((unsigned long long *)xs)[i] = h;
    if (c.vid == 0) stc_u64((unsigned long long *)st.norm_out + i, h);
  }
  __syncthreads();
}
// ... by the control wavefront of a tuned linear: lane l owns the 16-byte segments l, l + 64, ..., every segment lies in one part of
// the norm.  Weights and, where the previous stage does not write it, the residual row are requested before the barrier is awaited.
template <int KL>
__device__ __forceinline__ void mx_x_m1_prenorm_wave(CStage &st, Ctx &c, uint32_t *xs, int lane) {
  const f32x4 *w4 = (const f32x4 *)st.norm_w, *yw4 = (const f32x4 *)st.y_norm_w;
  const int ng = st.norm_groups, gl8 = st.k_real / ng / 8;
  f32x4 g[KL][2], x[KL][2], yw[KL][2];
  auto load_x = [&]() {
#pragma unroll
    for (int kc = 0; kc < KL; kc++)
#pragma unroll
      for (int h = 0; h < 2; h++) x[kc][h] = fx_ldc_quad((const float *)st.res + ((kc * 64 + lane) * 2 + h) * 4);
  };
#pragma unroll
  for (int kc = 0; kc < KL; kc++)
#pragma unroll
    for (int h = 0; h < 2; h++) {
      g[kc][h] = w4[(kc * 64 + lane) * 2 + h];
      yw[kc][h] = yw4 ? yw4[(kc * 64 + lane) * 2 + h] : (f32x4){1.f, 1.f, 1.f, 1.f};
    }
#if MK_HAVE_HYB
  f32x4 yb[KL][2];
#pragma unroll
  for (int kc = 0; kc < KL; kc++)
#pragma unroll
    for (int h = 0; h < 2; h++) yb[kc][h] = st.in_bias ? ((const f32x4 *)st.in_bias)[(kc * 64 + lane) * 2 + h] : (f32x4){0.f, 0.f, 0.f, 0.f};
#endif
  const bool early = st.flags & MK_F_RES_EARLY;
  if (early) load_x();
  if (c.pending && lane == 0) barrier_poll(c);
  if (!early) load_x();
  if (st.y_in) {
#if MK_HAVE_HYB
    f32x4 y[KL][2];
    if (st.slots == 0) {
      u32x4 raw[KL];
#pragma unroll
      for (int kc = 0; kc < KL; kc++) raw[kc] = ldc_16B((const u32x4 *)st.y_in + kc * 64 + lane);
#pragma unroll
      for (int kc = 0; kc < KL; kc++)
#pragma unroll
        for (int h = 0; h < 2; h++) {
          y[kc][h] = (f32x4){bf_lo(raw[kc][2 * h]), bf_hi(raw[kc][2 * h]), bf_lo(raw[kc][2 * h + 1]), bf_hi(raw[kc][2 * h + 1])};
          y[kc][h] += yb[kc][h];
        }
    } else {
#pragma unroll
      for (int kc = 0; kc < KL; kc++)
#pragma unroll
        for (int h = 0; h < 2; h++) y[kc][h] = (f32x4){0.f, 0.f, 0.f, 0.f};
      u32x4 raw[2][KL];
      float f[2];
      auto fetch = [&](int q, u32x4 (&r)[KL], float &g_) {
        const int at = min(q, st.slots - 1);
#pragma unroll
        for (int kc = 0; kc < KL; kc++) r[kc] = ldc_16B((const u32x4 *)((const uint16_t *)st.y_in + (size_t)at * st.ld_slot) + kc * 64 + lane);
        g_ = q < st.slots ? ldc_f32(st.slot_w + at) : 0.f;
      };
      for (int q = 0; q < st.slots; q += 2) {
        fetch(q, raw[0], f[0]);
        fetch(q + 1, raw[1], f[1]);
#pragma unroll
        for (int z = 0; z < 2; z++)
#pragma unroll
          for (int kc = 0; kc < KL; kc++)
#pragma unroll
            for (int h = 0; h < 2; h++)
              y[kc][h] += (f32x4){bf_lo(raw[z][kc][2 * h]), bf_hi(raw[z][kc][2 * h]), bf_lo(raw[z][kc][2 * h + 1]), bf_hi(raw[z][kc][2 * h + 1])} * f[z];
      }
    }
    auto ye = [&](int kc, int h, int e) { return y[kc][h][e]; };
#else
    u32x4 y[KL];
#pragma unroll
    for (int kc = 0; kc < KL; kc++) y[kc] = ldc_16B((const u32x4 *)st.y_in + kc * 64 + lane);
    auto ye = [&](int kc, int h, int e) { return (e & 1) ? bf_hi(y[kc][h * 2 + (e >> 1)]) : bf_lo(y[kc][h * 2 + (e >> 1)]); };
#endif
    float r = 1.f;
    if (yw4) {
      float ss = 0.f;
#pragma unroll
      for (int kc = 0; kc < KL; kc++)
#pragma unroll
        for (int e = 0; e < 8; e++) ss += ye(kc, e >> 2, e & 3) * ye(kc, e >> 2, e & 3);
      r = 1.f / sqrtf(wave_sum(ss) / (float)st.k_real + st.norm_eps);
    }
#pragma unroll
    for (int kc = 0; kc < KL; kc++)
#pragma unroll
      for (int h = 0; h < 2; h++)
#pragma unroll
        for (int e = 0; e < 4; e++) x[kc][h][e] = fmaf(st.alpha, (ye(kc, h, e) * r) * yw[kc][h][e], x[kc][h][e]);
  }
  float sq[KL], rk[KL];
#pragma unroll
  for (int kc = 0; kc < KL; kc++) {
    sq[kc] = rk[kc] = 0.f;
#pragma unroll
    for (int h = 0; h < 2; h++)
#pragma unroll
      for (int e = 0; e < 4; e++) sq[kc] += x[kc][h][e] * x[kc][h][e];
  }
  for (int q = 0; q < ng; q++) {
    float ss = 0.f;
#pragma unroll
    for (int kc = 0; kc < KL; kc++) ss += (kc * 64 + lane) / gl8 == q ? sq[kc] : 0.f;
    const float r = 1.f / sqrtf(wave_sum(ss) / (float)(gl8 * 8) + st.eps);
#pragma unroll
    for (int kc = 0; kc < KL; kc++)
      if ((kc * 64 + lane) / gl8 == q) rk[kc] = r;
  }
#pragma unroll
  for (int kc = 0; kc < KL; kc++) {
    u32x4 o16;
#pragma unroll
    for (int h = 0; h < 2; h++) {
      f32x4 o;
#pragma unroll
      for (int e = 0; e < 4; e++) o[e] = (x[kc][h][e] * rk[kc]) * g[kc][h][e];
      o16[h * 2] = pack2(o[0], o[1]);
      o16[h * 2 + 1] = pack2(o[2], o[3]);
      if (c.vid == 0 && st.out2) stc_16B((u32x4 *)st.out2 + (kc * 64 + lane) * 2 + h, __builtin_bit_cast(u32x4, x[kc][h]));
    }
    ((u32x4 *)xs)[kc * 64 + lane] = o16;
    if (c.vid == 0) stc_16B((u32x4 *)st.norm_out + kc * 64 + lane, o16);
  }
}

#if MK_HAVE_DUAL
// What a residual_prenorm with dual options does in front of a single-token linear, by the workgroup: v = res + alpha y_scale y + y2_scale y2,
// the normed row (norm_out, with a convolution: out3) and the linear's input row in LDS, which is the normed row or the sum of it and its convolution.  In two
// halves: whatever the previous stage does not write is requested before its barrier is awaited.  NS: quads per thread (0: none of this).
// One part of the norm; the norm weight, both factors and the convolution are optional as in the stage.
#define MX_EARLY_TAPS 4
template <int NS>
struct MxPrologue {
  f32x4 g[NS], x[NS], ys[NS], y2s[NS];
  unsigned long long cw[NS][MX_EARLY_TAPS], ring[NS][MX_EARLY_TAPS];
  int pos, k4;
  uint16_t *rows;
  __device__ __forceinline__ int at(int j) const { return min((int)threadIdx.x + j * MK_THREADS, k4 - 1); }
  __device__ __forceinline__ void load_x(CStage &st) {
#pragma unroll
    for (int j = 0; j < NS; j++) x[j] = fx_ldc_quad((const float *)st.res + 4 * at(j));
  }
  __device__ __forceinline__ void load(CStage &st, const Ctx &c) {
    k4 = st.k / 4;
    pos = __builtin_amdgcn_readfirstlane(c.sh_tok[0]);
    const f32x4 one = {1.f, 1.f, 1.f, 1.f};
#pragma unroll
    for (int j = 0; j < NS; j++) {
      g[j] = ((const f32x4 *)st.norm_w)[at(j)];
      ys[j] = st.y_scale ? ((const f32x4 *)st.y_scale)[at(j)] : one;
      y2s[j] = st.y2_scale ? ((const f32x4 *)st.y2_scale)[at(j)] : one;
    }
    if (st.conv_w) {
      const int taps = st.taps;
      rows = (uint16_t *)st.tail + (size_t)__builtin_amdgcn_readfirstlane(c.state_ids[__builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS])]) * taps * st.k;
#pragma unroll
      for (int b = 0; b < MX_EARLY_TAPS; b++) {
        const int back = min(b, taps - 1), row = max(pos - back, 0) % taps;
#pragma unroll
        for (int j = 0; j < NS; j++) {
          cw[j][b] = ((const unsigned long long *)((const uint16_t *)st.conv_w + (size_t)(taps - 1 - back) * st.k))[at(j)];
          if (b) ring[j][b] = ldc_u64(rows + (size_t)row * st.k + 4 * at(j));
        }
      }
    }
    if (st.flags & MK_F_RES_EARLY) load_x(st);
  }
  __device__ __forceinline__ void finish(CStage &st, const Ctx &c, uint32_t *xs, float *red) {
    auto quad = [](unsigned long long u) { return (f32x4){bf_lo((uint32_t)u), bf_hi((uint32_t)u), bf_lo((uint32_t)(u >> 32)), bf_hi((uint32_t)(u >> 32))}; };
    auto pack = [](f32x4 o) { return (unsigned long long)pack2(o[0], o[1]) | ((unsigned long long)pack2(o[2], o[3]) << 32); };
    const int tid = threadIdx.x;
    if (!(st.flags & MK_F_RES_EARLY)) load_x(st);
    if (st.y_in) {
      f32x4 y[NS], y2[NS];
      auto at_ = [&](int j) { return at(j); };
      mx_summands<uint16_t, NS>(st, (const uint16_t *)st.y_in, st.slot_w, st.slots && !st.y2, y, at_);
      if (st.y2) mx_summands<uint16_t, NS>(st, (const uint16_t *)st.y2, st.slot_w, st.slots, y2, at_);
#pragma unroll
      for (int j = 0; j < NS; j++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
          if (st.y2) x[j][e] = fmaf(y2s[j][e], y2[j][e], x[j][e]);
          x[j][e] = fmaf(st.alpha, y[j][e] * ys[j][e], x[j][e]);
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NS; j++)
      if (tid + j * MK_THREADS < k4) ss += x[j][0] * x[j][0] + x[j][1] * x[j][1] + x[j][2] * x[j][2] + x[j][3] * x[j][3];
    const float r = 1.f / sqrtf(block_sum(ss, red) / (float)st.k_real + st.eps);
#pragma unroll
    for (int j = 0; j < NS; j++) {
      const int i = tid + j * MK_THREADS;
      if (i >= k4) continue;
      unsigned long long hp = pack((x[j] * r) * g[j]);
      if (c.vid == 0) {
        if (st.out2) stc_16B((u32x4 *)st.out2 + i, __builtin_bit_cast(u32x4, x[j]));
        stc_u64((unsigned long long *)(st.conv_w ? st.out3 : st.norm_out) + i, hp);
        if (st.conv_w) stc_u64(rows + (size_t)(pos % st.taps) * st.k + 4 * i, hp);  // (a row nobody reads in this iteration)
      }
      if (st.conv_w) {
        const f32x4 h = quad(hp);
        f32x4 acc = h;
#pragma unroll
        for (int b = 0; b < MX_EARLY_TAPS; b++) {
          const f32x4 w = quad(cw[j][b]), v = b ? quad(ring[j][b]) : h;
#pragma unroll
          for (int e = 0; e < 4; e++) acc[e] = b < st.taps && b <= pos ? fmaf(v[e], w[e], acc[e]) : acc[e];
        }
        if (st.taps > MX_EARLY_TAPS) acc = mx_ring_conv<uint16_t>(st, rows, st.k, pos, i, MX_EARLY_TAPS, acc);
        hp = pack(acc);
      }
      ((unsigned long long *)xs)[i] = hp;
    }
    __syncthreads();
  }
};
template <> struct MxPrologue<0> {};
__device__ __forceinline__ bool mx_dual_prenorm(CStage &st) { return (st.flags & MK_F_PRENORM) && (st.y_scale || st.y2 || st.conv_w); }
#else
template <int NS> struct MxPrologue {};
__device__ __forceinline__ bool mx_dual_prenorm(CStage &) { return false; }
#endif

// ----------------------------------------------------------------------------- single-token linear, any reduction length
// out[n] = sum_k W[n, k] x[k], k a multiple of 64.  A wavefront owns a run of rows and takes R of them at a time, 512 U values of
// k per step, two steps' loads in flight; the first step's are requested before the previous stage's barrier is awaited (not by
// the wavefront that polls it).  MK_F_JOIN: the sum joins the residual stream, out2 = res + alpha * sum (32-bit), norm_out = the
// same rounded, and st.out is not written.
// PRO: the row comes from an MxPrologue of that many quads per thread (dual kernels; 0: it does not).
template <int R, int U, int PRO = 0>
__device__ __forceinline__ void stage_mx_linear_m1_t(CStage &st, Ctx &c, char *smem) {
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int K = st.k, k8 = K / 8, nkb = (k8 + 64 * U - 1) / (64 * U), n = st.n;
  u32x4 *xs4 = (u32x4 *)smem;
  const int nw = c.G * MK_WAVES, id = c.vid * MK_WAVES + wave, q = n / nw, rem = n - q * nw;
  const int r0 = id * q + min(id, rem), r1 = r0 + q + (id < rem ? 1 : 0);
  const int steps = ((r1 - r0 + R - 1) / R) * nkb;
  u32x4 A[R][U], B[R][U];
  auto load = [&](int step, u32x4 (&b)[R][U]) {
    const int rb = step / nkb, kb = step - rb * nkb;
#pragma unroll
    for (int r = 0; r < R; r++) {
      const u32x4 *w = weight_row(st.w, min(r0 + rb * R + r, n - 1), k8);
#pragma unroll
      for (int u = 0; u < U; u++) b[r][u] = ldg_stream(w + min((kb * U + u) * 64 + lane, k8 - 1));
    }
  };
  MxPrologue<PRO> pro;
  if constexpr (PRO > 0) {
    if (wave != 0) pro.load(st, c);
  }
  if (wave != 0) load(0, A);
  barrier_wait(c);
  for (int i = k8 + tid; i < nkb * U * 64; i += MK_THREADS) xs4[i] = (u32x4){0u, 0u, 0u, 0u};  // (nothing multiplies the repeated loads)
  if constexpr (PRO > 0) {
    if (wave == 0) pro.load(st, c);
    pro.finish(st, c, (uint32_t *)smem, (float *)(smem + MK_RED_OFFSET));
  } else {
    stage_x_m1<true>(st, c, (uint32_t *)smem, (float *)(smem + MK_RED_OFFSET));
  }
  if (wave == 0) load(0, A);
  const bool join = st.flags & MK_F_JOIN;
  float acc[R];
#pragma unroll
  for (int r = 0; r < R; r++) acc[r] = 0.f;
  auto consume = [&](int step, const u32x4 (&b)[R][U]) {
    const int rb = step / nkb, kb = step - rb * nkb;
#pragma unroll
    for (int u = 0; u < U; u++) {
      const u32x4 x = xs4[(kb * U + u) * 64 + lane];
#pragma unroll
      for (int r = 0; r < R; r++) acc[r] = dot8(b[r][u], x, acc[r]);
    }
    if (kb + 1 < nkb) return;
    const int row = r0 + rb * R + lane;
    const bool mine = lane < R && row < r1;
    const float x = join && mine ? ldc_f32((const float *)st.res + row) : 0.f;
    float v = 0.f;
#pragma unroll
    for (int r = 0; r < R; r++) {
      const float s = wave_sum(acc[r]);
      v = lane == r ? s : v;
      acc[r] = 0.f;
    }
    if (mine) {
      if (join) {
        v = fmaf(st.alpha, v, x);
        stc_f32((float *)st.out2 + row, v);
        stc_u16((uint16_t *)st.norm_out + row, (uint16_t)f2bf(v));
      } else {
        stc_u16((uint16_t *)st.out + row, (uint16_t)f2bf(linear_act(st, v)));
      }
    }
  };
  for (int s = 0; s < steps; s += 2) {
    load(min(s + 1, steps - 1), B);
    consume(s, A);
    if (s + 1 >= steps) break;
    load(min(s + 2, steps - 1), A);
    consume(s + 1, B);
  }
  c.wrote_through = true;
}
// (which single-token linears: those that join the stream, and those no tuned instantiation exists for)
__device__ __forceinline__ bool mx_linear_m1_form(CStage &st) {
  return !(st.flags & (MK_F_SILU | MK_F_RES)) && (st.k & 63) == 0 && ((st.flags & MK_F_JOIN) || mx_dual_prenorm(st) || (st.k != 4096 && st.k != 2048 && st.k != 1024 && st.k != 12288));
}
__device__ __forceinline__ void stage_mx_linear_m1(CStage &st, Ctx &c, char *smem) {
#if MK_HAVE_DUAL
  if (mx_dual_prenorm(st)) {
    if (st.k <= 1024) stage_mx_linear_m1_t<4, 2, 1>(st, c, smem);
    else if (st.k <= 4 * 4 * MK_THREADS) stage_mx_linear_m1_t<4, 4, 4>(st, c, smem);
    else stage_mx_linear_m1_t<4, 4, 12>(st, c, smem);
    return;
  }
#endif
  if (st.k <= 512) stage_mx_linear_m1_t<4, 1>(st, c, smem);
  else if (st.k <= 1536) stage_mx_linear_m1_t<4, 3>(st, c, smem);
  else stage_mx_linear_m1_t<4, 4>(st, c, smem);
}

// ----------------------------------------------------------------------------- gated activation
// Elements of the rows, 1024 per item, dealt from the last workgroup downwards (the stage's own units start at the first).
template <typename E>
__device__ __forceinline__ void mx_glu(CStage &st, Ctx &c, int M) {
  if (!st.glu_out) return;
  const int n = st.glu_n, per = (n + 4 * MK_THREADS - 1) / (4 * MK_THREADS), total = M * per;
  const float lim = st.glu_limit, beta = st.glu_beta, bias = st.glu_bias;
  for (int i = c.G - 1 - mx_spread(c); i < total; i += c.G) {
    const int t = i / per, d = (i - t * per) * 4 * MK_THREADS + 4 * threadIdx.x;
    if (d >= n) continue;
    const E *row = (const E *)st.in + (size_t)t * st.ld_in;
    const f32x4 a = fx_ldc_quad(row + st.glu_gate + d), b = fx_ldc_quad(row + st.glu_up + d);
    f32x4 o;
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const float g = fminf(a[e], lim), u = fminf(fmaxf(b[e], -lim), lim);
      o[e] = g * mx_sigmoid(E(), beta * g) * (u + bias);
    }
    fx_stc_quad((E *)st.glu_out + (size_t)t * st.ld_glu + d, o);
  }
}

// ----------------------------------------------------------------------------- latent rows
// One wavefront: row of n values (n4 quads are readable, those behind n are zero) / rms * w; put(quad index, values).  NQ: quads
// per lane, 256 NQ >= n; every load is unconditional (indices are clamped), so all of them are in flight together.
template <typename E, int NQ, typename Put>
__device__ __forceinline__ void mx_norm_row_t(const E *src, const float *w, int n, float eps, int lane, Put put) {
  const int n4 = (n + 3) / 4;
  f32x4 v[NQ], g[NQ];
#pragma unroll
  for (int j = 0; j < NQ; j++) v[j] = fx_ldc_quad(src + 4 * min(j * 64 + lane, n4 - 1));
#pragma unroll
  for (int j = 0; j < NQ; j++) g[j] = ((const f32x4 *)w)[min(j * 64 + lane, n4 - 1)];
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NQ; j++) {
    const float q = v[j][0] * v[j][0] + v[j][1] * v[j][1] + v[j][2] * v[j][2] + v[j][3] * v[j][3];
    ss += j * 64 + lane < n4 ? q : 0.f;
  }
  const float r = 1.f / sqrtf(wave_sum(ss) / (float)n + eps);
#pragma unroll
  for (int j = 0; j < NQ; j++)
    if (j * 64 + lane < n4) put(j * 64 + lane, (v[j] * r) * g[j]);
}
template <typename E, typename Put>
__device__ __forceinline__ void mx_norm_row(const E *src, const float *w, int n, float eps, int lane, Put put) {
  if (n <= 512) mx_norm_row_t<E, 2>(src, w, n, eps, lane, put);
  else if (n <= 2048) mx_norm_row_t<E, 8>(src, w, n, eps, lane, put);
  else mx_norm_row_t<E, MK_MX_MAX_NORM_ROW / 256>(src, w, n, eps, lane, put);
}
// A cached latent: the normalised latent, padded with zeros to whole operand rows, then the rotated key part, padded likewise.
// Inside a page: [position / 16][operand row][64 lanes][EPC], lane l holds position l % 16, dims (l / 16) * EPC .. of the row.
template <typename E>
__device__ __forceinline__ size_t mx_latent_at(int page, int pp, int ps, int nkc, int d) { return fx_k_at<E>(page, pp, ps, 1, 0, nkc, d); }

template <typename E>
__device__ __forceinline__ void stage_mx_latent_prep(CStage &st, Ctx &c, const MkRuntime &rt, int M) {
  barrier_wait(c);
  constexpr int KW = FxType<E>::KW;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int R = st.rank, rot = st.rot_dims, half = rot / 2, nrc = (R + KW - 1) / KW, nkc = nrc + (rot + KW - 1) / KW, ps = rt.page_size;
  const int nq = st.n > 0, per = nq + (st.k_cache ? 1 : 0), total = M * per;  // (a model may form its queries without a latent)
  for (int i = mx_wave_item(c, wave); i < total; i += c.G * MK_WAVES) {
    const int t = i / per;
    const E *row = (const E *)st.in + (size_t)t * st.ld_in;
    if (i - t * per < nq) {
      E *o = (E *)st.out + (size_t)t * st.ld_out;
      mx_norm_row<E>(row + st.cols[0], (const float *)st.q_norm_w, st.n, st.eps, lane, [&](int q, f32x4 v) { fx_stc_quad(o + 4 * q, v); });
    } else {
      const int pos = __builtin_amdgcn_readfirstlane(c.sh_tok[t]), pp = pos % ps;
      const int page = rt.kv_indices[__builtin_amdgcn_readfirstlane(c.sh_tok[3 * MK_MAX_TOKENS + t]) + pos / ps];
      E *kc = (E *)st.k_cache;
      mx_norm_row<E>(row + st.cols[1], (const float *)st.k_norm_w, R, st.eps, lane,
                     [&](int q, f32x4 v) { fx_stc_quad(kc + mx_latent_at<E>(page, pp, ps, nkc, 4 * q), v); });
      for (int q = (R + 3) / 4 + lane; q < nrc * KW / 4; q += 64) fx_stc_quad(kc + mx_latent_at<E>(page, pp, ps, nkc, 4 * q), (f32x4){0.f, 0.f, 0.f, 0.f});
      const E *kr = row + st.cols[2];
      const float *ct = (const float *)st.cos_tab + (size_t)pos * st.ld_cos, *sn = (const float *)st.sin_tab + (size_t)pos * st.ld_cos;
      for (int d = lane; d < (nkc - nrc) * KW; d += 64) {
        float v = 0.f;
        if (d < rot) {
          const int f = d < half ? d : d - half;
          const float x = fx_ldc(kr + d), y = fx_ldc(kr + (d < half ? d + half : f));
          v = d < half ? x * ct[f] - y * sn[f] : x * ct[f] + y * sn[f];
        }
        fx_stc(kc + mx_latent_at<E>(page, pp, ps, nkc, nrc * KW + d), fx_round<E>(v));
      }
    }
  }
  mx_glu<E>(st, c, M);
  c.wrote_through = true;
}

// ----------------------------------------------------------------------------- a matrix per head
// out[t, h * ld_out_slot + n] = sum_k in[t, h * ld_in_slot + k] W[h][n][k],  n < st.n,  k < st.k (whole operand rows).  Weights
// are [head][n / 16][k / KW][64 lanes][EPC]: lane l holds row l % 16, k (l / 16) * EPC .. .  A wavefront per 16-row tile and all
// tokens; few tiles with long rows: a workgroup per tile and 16 tokens, its wavefronts split K.
//   MX_GELU:   out = gelu(sum) * table[id(t)][n]
//   MX_OUT32:  out2 = sum in 32 bits
//   MX_STEP:   out2 = softplus(sum + in_bias[n]) in 32 bits
//   MX_DECAY:  tanh is applied to the inputs (kept as value + remainder in bf16), out2 = exp(-exp(-1/2) sigmoid(sum + offset[n]))
//              in 32 bits, and the gated activation runs beside it
enum { MX_PLAIN, MX_GELU, MX_DECAY, MX_OUT32, MX_STEP };
template <typename E, int MT, int EPI, bool SPLIT>
__device__ __forceinline__ void stage_mx_head_linear_t(CStage &st, Ctx &c, int M, char *smem) {
  constexpr int EPC = FxType<E>::EPC, KW = FxType<E>::KW, KB = MT == 4 ? 4 : SPLIT ? 16 : EPI == MX_DECAY ? 4 : 8, B16 = sizeof(E) == 2;
  static_assert(!SPLIT || MT == 1, "");
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int N = st.n, nks = st.k / KW, nt = (N + 15) / 16, mts = MT == 1 ? (M + 15) / 16 : 1, items = st.groups * nt * mts;
  const int kq = SPLIT ? (nks + MK_WAVES - 1) / MK_WAVES : nks;
  const int kb = SPLIT ? min(nks, wave * kq) : 0, ke = SPLIT ? min(nks, kb + kq) : nks;
  const u32x4 *W = (const u32x4 *)st.w.seg[0];
  const int i0 = SPLIT ? mx_spread(c) : mx_wave_item(c, wave), di = SPLIT ? c.G : c.G * MK_WAVES;
  f32x4 *red = (f32x4 *)smem;
  const u32x4 zero = {0u, 0u, 0u, 0u};
  u32x4 a[KB];
  auto load_w = [&](int i, int k0) {
#pragma unroll
    for (int j = 0; j < KB; j++) a[j] = ldg_stream(W + ((size_t)(i / mts) * nks + min(k0 + j, nks - 1)) * 64 + lane);
  };
  // weights do not depend on the previous stage: the first tile's are requested before its barrier completes
  const bool early = i0 < items && wave != 0;
  if (early) load_w(i0, kb);
  if (tid == 0) __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
  barrier_wait(c);
  for (int i = i0; i < items; i += di) {
    const int tile = i / mts, mt0 = i - tile * mts, h = tile / nt, n0 = (tile - h * nt) * 16 + lg * 4;
    const E *xr[MT];
#pragma unroll
    for (int m = 0; m < MT; m++) xr[m] = (const E *)st.in + (size_t)min((mt0 + m) * 16 + lr, M - 1) * st.ld_in + (size_t)h * st.ld_in_slot + lg * EPC;
    f32x4 acc[MT];
#pragma unroll
    for (int m = 0; m < MT; m++) acc[m] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int k0 = kb; k0 < ke; k0 += KB) {
      if (!(early && i == i0 && k0 == kb)) load_w(i, k0);
      u32x4 b[KB][MT];
#pragma unroll
      for (int j = 0; j < KB; j++)
#pragma unroll
        for (int m = 0; m < MT; m++) b[j][m] = *(const u32x4 *)(xr[m] + (size_t)min(k0 + j, nks - 1) * KW);
#pragma unroll
      for (int j = 0; j < KB; j++) {
        const u32x4 w = k0 + j < ke ? a[j] : zero;
#pragma unroll
        for (int m = 0; m < MT; m++) {
          if constexpr (EPI == MX_DECAY) {
            u32x4 hi, lo;
#pragma unroll
            for (int q = 0; q < 4; q++) {
              if constexpr (B16) {
                const float x0 = mx_tanh(E(), bf_lo(b[j][m][q])), x1 = mx_tanh(E(), bf_hi(b[j][m][q]));
                hi[q] = pack2(x0, x1);
                lo[q] = pack2(x0 - bf_lo(hi[q]), x1 - bf_hi(hi[q]));
              } else {
                hi[q] = __float_as_uint(mx_tanh(E(), __uint_as_float(b[j][m][q])));
              }
            }
            acc[m] = fx_mma_k(E(), w, hi, acc[m]);
            if constexpr (B16) acc[m] = fx_mma_k(E(), w, lo, acc[m]);
          } else {
            acc[m] = fx_mma_k(E(), w, b[j][m], acc[m]);
          }
        }
      }
    }
    if constexpr (SPLIT) {
      __syncthreads();
      red[wave * 64 + lane] = acc[0];
      __syncthreads();
      if (wave != 0) continue;
      acc[0] = red[lane] + red[64 + lane] + red[128 + lane] + red[192 + lane];
    }
#pragma unroll
    for (int m = 0; m < MT; m++) {
      const int t = (mt0 + m) * 16 + lr;
      if (t >= M) continue;
      float r[4] = {acc[m][0], acc[m][1], acc[m][2], acc[m][3]};
      if constexpr (EPI == MX_GELU) {
        const long long id = (long long)ldc_u64((const long long *)st.aux0 + t);
        const E *e = (const E *)st.aux1 + (size_t)(id < 0 ? 0 : id) * st.ld_res;
        float f[4];
#pragma unroll
        for (int q = 0; q < 4; q++) f[q] = fx_val(e[min(n0 + q, N - 1)]);
#pragma unroll
        for (int q = 0; q < 4; q++) {
          const float z = r[q], th = mx_tanh(E(), 0.7978845608028654f * (z + 0.044715f * z * z * z));
          r[q] = id < 0 ? 0.f : 0.5f * z * (1.f + th) * f[q];
        }
      }
      if constexpr (EPI == MX_DECAY) {
        const f32x4 w0 = *(const f32x4 *)((const float *)st.q_norm_w + n0);
        f32x4 d;
#pragma unroll
        for (int q = 0; q < 4; q++) d[q] = expf(-0.6065306597126334f * mx_sigmoid(E(), r[q] + w0[q]));
        fx_stc_quad((float *)st.out2 + (size_t)t * st.ld_out2 + n0, d);
#if MK_HAVE_HYB
      } else if constexpr (EPI == MX_OUT32) {
        fx_stc4((float *)st.out2 + (size_t)t * st.ld_out2, n0, N, r);
      } else if constexpr (EPI == MX_STEP) {
        const f32x4 b = *(const f32x4 *)(st.in_bias + n0);
        f32x4 d;
#pragma unroll
        for (int q = 0; q < 4; q++) {
          const float z = r[q] + b[q];
          d[q] = z > 20.f ? z : log1pf(expf(z));
        }
        fx_stc_quad((float *)st.out2 + (size_t)t * st.ld_out2 + n0, d);
#endif
      } else {
        fx_stc4((E *)st.out + (size_t)t * st.ld_out + (size_t)h * st.ld_out_slot, n0, N, r);
      }
    }
  }
  if constexpr (EPI == MX_DECAY) mx_glu<E>(st, c, M);
  c.wrote_through = true;
}
template <typename E, int MAXM>
__device__ __forceinline__ void stage_mx_head_linear(CStage &st, Ctx &c, int M, char *smem) {
#if MK_HAVE_HYB
  if (st.flags & MK_F_OUT32) {
    if (st.groups * ((st.n + 15) / 16) * 4 <= c.G && st.k / FxType<E>::KW >= 8) stage_mx_head_linear_t<E, 1, MX_OUT32, true>(st, c, M, smem);
    else stage_mx_head_linear_t<E, 1, MX_OUT32, false>(st, c, M, smem);
    return;
  }
#endif
  if (st.groups * ((st.n + 15) / 16) * 4 <= c.G && st.k / FxType<E>::KW >= 8) {
    if (st.flags & MK_F_GELU_TABLE) stage_mx_head_linear_t<E, 1, MX_GELU, true>(st, c, M, smem);
    else stage_mx_head_linear_t<E, 1, MX_PLAIN, true>(st, c, M, smem);
  } else if (st.flags & MK_F_GELU_TABLE) {
    stage_mx_head_linear_t<E, 1, MX_GELU, false>(st, c, M, smem);
  } else if (MAXM == 1 || st.groups * ((st.n + 15) / 16) * ((M + 15) / 16) <= MK_WAVES * c.G) {
    stage_mx_head_linear_t<E, 1, MX_PLAIN, false>(st, c, M, smem);
  } else {
    stage_mx_head_linear_t<E, 4, MX_PLAIN, false>(st, c, M, smem);
  }
}

// ----------------------------------------------------------------------------- latent attention
// Scores are q' . c + q_rot . k_rot with q' the head's query carried into the latent space, results are sums of latents: one
// cached row per position serves every head as key and as value.  Query row = (token, head), tokens outermost.
//
// Work unit = 16 RT query rows of one request x a chunk of its cached tiles of 16 SUB positions.  The workgroup stages a tile
// in LDS in operand order (requested one tile ahead, so it is in flight while the previous one is used).  Wavefront s forms
// the scores of sub-tile s; maxima and weights are exchanged through LDS; then every wavefront takes every fourth 16-wide block
// of the latent over all positions, reading it from the same LDS tile transposed.  Weights enter as value + remainder in bf16.
struct MxLatentRows {
  int my_n, my_tiles, tiles_incl, total, cmax;
};
__device__ __forceinline__ MxLatentRows mx_latent_rows(const Ctx &c, int M, int H, int unit_rows) {
  const int lane = threadIdx.x & 63;
  MxLatentRows r;
  const bool first = lane < M && c.sh_tok[2 * MK_MAX_TOKENS + lane] == lane;
  const unsigned long long fm = __ballot(first), later = lane < 63 ? fm >> (lane + 1) : 0ull;
  r.my_n = first ? (later ? (int)__ffsll(later) : M - lane) : 0;
  r.my_tiles = (r.my_n * H + unit_rows - 1) / unit_rows;
  r.tiles_incl = wave_incl_scan(r.my_tiles, lane);
  r.total = wave_bcast(r.tiles_incl, 63);
  r.cmax = max(1, min(c.G / r.total, MK_MX_MAX_CHUNKS));
  return r;
}
// Chunks of a unit with NT tiles.
__device__ __forceinline__ int mx_chunks(int NT, int cmax) { return NT <= 2 ? 1 : min(cmax, NT); }

// 16-wide block of the latent, transposed out of the LDS tile: lane l gets dim l % 16 of the block at positions 4 (l / 16) .. + 3
// of sub-tiles s and s + 1 (bf16) or of sub-tile s (32-bit).
typedef short mx_s4 __attribute__((ext_vector_type(4)));
__device__ __forceinline__ u32x4 mx_value_operand(uint16_t, const char *kt, int nkc, int s, int b, int lane) {
  // the transposing read works on 16 lanes at a time: they address four rows of 16 values, four values each, and receive a
  // column of four
  const int lr = lane & 15, lg = lane >> 4;
  const char *p = kt + (s * nkc + (b >> 1)) * 1024 + (b & 1) * 512 + (((lr & 3) >> 1) * 16 + lg * 4 + (lr >> 2)) * 16 + (lr & 1) * 8;
  typedef __attribute__((address_space(3))) mx_s4 lds_s4;
  const mx_s4 x = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4 *)p), y = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s4 *)(p + nkc * 1024));
  typedef unsigned u32x2 __attribute__((ext_vector_type(2)));
  const u32x2 xx = __builtin_bit_cast(u32x2, x), yy = __builtin_bit_cast(u32x2, y);
  return (u32x4){xx[0], xx[1], yy[0], yy[1]};
}
__device__ __forceinline__ u32x4 mx_value_operand(float, const char *kt, int nkc, int s, int b, int lane) {
  const int lr = lane & 15, lg = lane >> 4;
  const unsigned *p = (const unsigned *)(kt + (s * nkc + b) * 1024) + ((lr >> 2) * 16 + lg * 4) * 4 + (lr & 3);
  return (u32x4){p[0], p[4], p[8], p[12]};
}

// NK: operand rows of a cached latent the instantiation has room for (rows behind the real ones repeat one and meet zeros in the
// query), SUB: sub-tiles per tile, VBW: 16-wide blocks per wavefront, RT: 16-row query tiles.  No loop of the tile walk has a
// run-time bound or a branch, so that its loads and LDS reads are scheduled together.
template <typename E, int NK, int SUB, int VBW, int RT>
__device__ __forceinline__ void stage_mx_latent_attn_t(CStage &st, Ctx &c, const MkRuntime &rt, int M, char *smem) {
  using X = FxType<E>;
  constexpr int EPC = X::EPC, KW = X::KW, B16 = sizeof(E) == 2, TPOS = 16 * SUB, PARTS = MK_WAVES / SUB, KC = (NK + PARTS - 1) / PARTS;
  constexpr int QN = RT * NK * 64 / MK_THREADS, GRP = NK % 6 == 0 ? 6 : 5;
  static_assert(RT * NK % 4 == 0, "whole rounds of query operands");
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int H = st.num_q_heads, R = st.rank, rot = st.rot_dims, half = rot / 2;
  const int nrc = (R + KW - 1) / KW, npc = (rot + KW - 1) / KW, nkc = nrc + npc, nvb = nrc * KW / 16, Rp = nrc * KW, PST = Rp + 32;
  const int ps = rt.page_size;
  const int my_sub = wave % SUB, my_part = wave / SUB;
  const MkLatentLds L = mk_latent_lds(sizeof(E), RT, NK, SUB, 0);
  u32x4 *qs = (u32x4 *)smem;
  char *kt = smem + L.kt;
  u32x4 *pb = (u32x4 *)(smem + L.pb);
  float *mx = (float *)(smem + L.mx), *ls = mx + 4 * RT * 16;
  int *spg = (int *)(smem + L.pages);
  const u32x4 *kc = (const u32x4 *)st.k_cache;
  const MxLatentRows rw = mx_latent_rows(c, M, H, 16 * RT);
  const int cmax = rw.cmax, n_units = rw.total * cmax;
  {  // (every workgroup: will some request be split?  then the merge stage runs)
    const int NT = rw.my_n ? (c.sh_tok[lane] + rw.my_n - 1) / TPOS + 1 : 0;
    c.mx_split = __any(rw.my_n && mx_chunks(NT, cmax) > 1);
  }
  struct Unit {
    int item, cidx, C, t0, r0, nrows, p0, p, tb, te, pages;
  };
  auto decode = [&](int u, Unit &a) -> bool {
    a.item = u / cmax;
    a.cidx = u - a.item * cmax;
    a.t0 = (int)__ffsll(__ballot(rw.tiles_incl > a.item)) - 1;
    const int n = wave_bcast(rw.my_n, a.t0);
    a.r0 = (a.item - (wave_bcast(rw.tiles_incl, a.t0) - wave_bcast(rw.my_tiles, a.t0))) * 16 * RT;
    a.nrows = min(16 * RT, n * H - a.r0);
    a.p0 = __builtin_amdgcn_readfirstlane(c.sh_tok[a.t0]);
    a.p = a.p0 + (a.r0 + a.nrows - 1) / H;  // newest position any of the rows sees
    // (chunks by the request's newest position, so that the merge stage finds the same count; a chunk that begins behind
    // this unit's own newest position contributes nothing)
    const int NT = (a.p0 + n - 1) / TPOS + 1;
    a.C = mx_chunks(NT, cmax);
    if (a.cidx >= a.C) return false;
    a.tb = (int)(((long long)NT * a.cidx) / a.C);
    a.te = min((int)(((long long)NT * (a.cidx + 1)) / a.C), a.p / TPOS + 1);
    a.pages = __builtin_amdgcn_readfirstlane(c.sh_tok[3 * MK_MAX_TOKENS + a.t0]);
    return true;
  };
  u32x4 kv[KC];
  auto load_tile = [&](int tile, int page) {
    const int pp = (tile * TPOS) % ps;
    const u32x4 *p = kc + ((((size_t)page * ps + pp) / 16 + my_sub) * nkc) * 64 + lane;
#pragma unroll
    for (int j = 0; j < KC; j++) kv[j] = p[min(j * PARTS + my_part, nkc - 1) * 64];
  };
  auto store_tile = [&](int tile, int newest) {
    const bool hidden = tile * TPOS + my_sub * 16 + lr > newest;  // rows behind the newest position belong to nobody
    u32x4 *dst = (u32x4 *)kt + (my_sub * NK + my_part) * 64 + lane;
#pragma unroll
    for (int j = 0; j < KC; j++) dst[j * PARTS * 64] = hidden ? (u32x4){0u, 0u, 0u, 0u} : kv[j];
  };
  Unit a0;
  const int u0 = mx_spread(c);
  const bool have0 = u0 < n_units && decode(u0, a0);
  // the first tile is requested before the barrier is awaited when earlier iterations wrote all of it
  const bool early = have0 && wave != 0 && a0.tb < a0.te && (a0.tb + 1) * TPOS <= a0.p0;
  if (early) load_tile(a0.tb, rt.kv_indices[a0.pages + a0.tb * TPOS / ps]);
  if (tid == 0) __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");  // rows of this iteration are read with cached loads
  barrier_wait(c);
  const float sc1 = st.sm_scale * 1.4426950408889634f;
  for (int u = u0; u < n_units; u += c.G) {
    Unit a;
    if (u == u0) {
      if (!have0) continue;
      a = a0;
    } else if (!decode(u, a)) {
      continue;
    }
    if (a.tb < a.te && !(u == u0 && early)) load_tile(a.tb, rt.kv_indices[a.pages + a.tb * TPOS / ps]);
    __syncthreads();  // LDS reuse across units
    const int pg_lo = a.tb * TPOS / ps, npg = a.tb + 1 < a.te ? (a.te * TPOS - 1) / ps - pg_lo + 1 : 0;  // (pages of the tiles behind the first)
    for (int i = tid; i < npg; i += MK_THREADS) spg[i] = rt.kv_indices[a.pages + min(pg_lo + i, a.p / ps)];
    // ---- query rows in operand order: latent parts, and (in the zeros left for it) the rotated part.  A wavefront takes every
    // fourth operand row, so which one it is and where it goes are scalars; a lane always has the same query row of a row tile.
    {
      const E *ql[RT], *qr[RT];
      const float *ct[RT], *sn[RT];
      bool real[RT];
#pragma unroll
      for (int q = 0; q < RT; q++) {
        const int r = q * 16 + lr, Rw = a.r0 + min(r, a.nrows - 1), t = a.t0 + Rw / H, h = Rw % H, pos = c.sh_tok[t];
        real[q] = r < a.nrows;
        ql[q] = (const E *)st.q_ws + (size_t)t * st.ld_qws + (size_t)h * Rp + lg * EPC;
        qr[q] = (const E *)st.in + (size_t)t * st.ld_in + (size_t)h * st.ld_in_slot + st.cols[0];
        ct[q] = (const float *)st.cos_tab + (size_t)pos * st.ld_cos;
        sn[q] = (const float *)st.sin_tab + (size_t)pos * st.ld_cos;
      }
      u32x4 v[QN];
#pragma unroll
      for (int k = 0; k < QN; k++) {
        const int rc = wave + k * MK_WAVES, q = rc >= NK, ch = rc - q * NK;
        v[k] = ldc_16B((const u32x4 *)(ql[RT == 1 ? 0 : q] + min(ch, nrc - 1) * KW));
      }
      // parts of 16-byte words: dims d0 .. of the rotated part and their partners half a part away
      if ((half % EPC) == 0) {
        for (int rc = wave; rc < RT * npc; rc += MK_WAVES) {
          const int q = rc >= npc, d0 = (rc - q * npc) * KW + lg * EPC, dc = min(d0, rot - EPC), k0 = dc < half ? dc : dc - half;
          const E *x = qr[RT == 1 ? 0 : q];
          const float *cs = ct[RT == 1 ? 0 : q] + k0, *sv = sn[RT == 1 ? 0 : q] + k0;
          const f32x4 x0 = fx_ldc_quad(x + dc), y0 = fx_ldc_quad(x + (dc < half ? dc + half : k0)), c0 = *(const f32x4 *)cs, s0 = *(const f32x4 *)sv;
          f32x4 x1, y1, c1, s1;
          if constexpr (B16) {
            x1 = fx_ldc_quad(x + dc + 4);
            y1 = fx_ldc_quad(x + (dc < half ? dc + half : k0) + 4);
            c1 = *(const f32x4 *)(cs + 4);
            s1 = *(const f32x4 *)(sv + 4);
          }
          const float sgn = dc < half ? -1.f : 1.f;
          const bool on = d0 < rot && real[RT == 1 ? 0 : q];
          u32x4 w;
#pragma unroll
          for (int e = 0; e < 4; e++) {
            const float z0 = on ? fmaf(sgn * y0[e], s0[e], x0[e] * c0[e]) : 0.f;
            if constexpr (B16) {
              const float z1 = on ? fmaf(sgn * y1[e], s1[e], x1[e] * c1[e]) : 0.f;
              ((uint16_t *)&w)[e] = (uint16_t)f2bf(z0);
              ((uint16_t *)&w)[4 + e] = (uint16_t)f2bf(z1);
            } else {
              w[e] = __float_as_uint(z0);
            }
          }
          qs[(q * NK + nrc + rc - q * npc) * 64 + lane] = w;
        }
      } else {
        for (int rc = wave; rc < RT * npc; rc += MK_WAVES) {
          const int q = rc >= npc;
          E *dst = (E *)(qs + (q * NK + nrc + rc - q * npc) * 64 + lane);
#pragma unroll 1
          for (int e = 0; e < EPC; e++) {
            const int d = (rc - q * npc) * KW + lg * EPC + e, dc = min(d, rot - 1), k = dc < half ? dc : dc - half;
            const E *x = qr[RT == 1 ? 0 : q];
            const float xv = fx_ldc(x + dc), yv = fx_ldc(x + (dc < half ? dc + half : k)), cv = ct[RT == 1 ? 0 : q][k], sv = sn[RT == 1 ? 0 : q][k];
            dst[e] = fx_round<E>(d < rot && real[RT == 1 ? 0 : q] ? (dc < half ? xv * cv - yv * sv : xv * cv + yv * sv) : 0.f);
          }
        }
      }
#pragma unroll
      for (int k = 0; k < QN; k++) {
        const int rc = wave + k * MK_WAVES, q = rc >= NK, ch = rc - q * NK;
        const bool on = ch < nrc && real[RT == 1 ? 0 : q];
        if (ch < nrc || ch >= nkc) qs[rc * 64 + lane] = on ? v[k] : (u32x4){0u, 0u, 0u, 0u};
      }
    }
    MK_MARK(c, 0);
    // ---- tiles
    int plim[RT];
    float m[RT], l[RT];
    f32x4 acc[RT][VBW];
#pragma unroll
    for (int q = 0; q < RT; q++) {
      plim[q] = a.p0 + (a.r0 + min(q * 16 + lr, a.nrows - 1)) / H;  // newest position this lane's query row sees
      m[q] = MK_FX_NEG;
      l[q] = 0.f;
#pragma unroll
      for (int b = 0; b < VBW; b++) acc[q][b] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
    for (int tile = a.tb; tile < a.te; tile++) {
      __syncthreads();  // the previous tile has been read (first tile: queries and pages are in place)
      store_tile(tile, a.p);
      if (tile + 1 < a.te) load_tile(tile + 1, spg[(tile + 1) * TPOS / ps - pg_lo]);
      __syncthreads();
      float sc[RT][4];
      if (SUB == MK_WAVES || wave < SUB) {
        f32x4 S[RT][2];  // (two chains per row tile)
#pragma unroll
        for (int q = 0; q < RT; q++) S[q][0] = S[q][1] = (f32x4){0.f, 0.f, 0.f, 0.f};
        // (operands are fetched a group at a time and held back from the products: left alone they are fetched one by one)
#pragma unroll
        for (int c0 = 0; c0 < NK; c0 += GRP) {
          u32x4 k[GRP], b[RT][GRP];
#pragma unroll
          for (int y = 0; y < GRP; y++) {
            k[y] = ((const u32x4 *)kt)[(wave * NK + c0 + y) * 64 + lane];
#pragma unroll
            for (int q = 0; q < RT; q++) b[q][y] = qs[(q * NK + c0 + y) * 64 + lane];
          }
          __builtin_amdgcn_sched_barrier(0);
#pragma unroll
          for (int y = 0; y < GRP; y++)
#pragma unroll
            for (int q = 0; q < RT; q++) S[q][y & 1] = fx_mma_k(E(), k[y], b[q][y], S[q][y & 1]);
        }
#pragma unroll
        for (int q = 0; q < RT; q++) {
          const f32x4 s = S[q][0] + S[q][1];
          float tm = MK_FX_NEG;
#pragma unroll
          for (int i = 0; i < 4; i++) {
            sc[q][i] = tile * TPOS + wave * 16 + lg * 4 + i <= plim[q] ? s[i] * sc1 : MK_FX_NEG;
            tm = fmaxf(tm, sc[q][i]);
          }
          tm = groups_max(tm);
          if (lg == 0) mx[(wave * RT + q) * 16 + lr] = tm;
        }
      }
      __syncthreads();
      float nm[RT];
      bool grow = false;
#pragma unroll
      for (int q = 0; q < RT; q++) {
        nm[q] = m[q];
#pragma unroll
        for (int s = 0; s < SUB; s++) nm[q] = fmaxf(nm[q], mx[(s * RT + q) * 16 + lr]);
        grow = grow || nm[q] > m[q];
      }
      if (__any(grow)) {
#pragma unroll
        for (int q = 0; q < RT; q++) {
          const float corr = fx_exp2(E(), m[q] - nm[q]);
          m[q] = nm[q];
          l[q] *= corr;
#pragma unroll
          for (int b = 0; b < VBW; b++) acc[q][b] *= corr;
        }
      }
      if (SUB == MK_WAVES || wave < SUB) {
#pragma unroll
        for (int q = 0; q < RT; q++) {
#pragma unroll
          for (int i = 0; i < 4; i++) {
            sc[q][i] = sc[q][i] > 0.5f * MK_FX_NEG ? fx_exp2(E(), sc[q][i] - m[q]) : 0.f;
            l[q] += sc[q][i];
          }
          if constexpr (B16) {
            const uint32_t h0 = pack2(sc[q][0], sc[q][1]), h1 = pack2(sc[q][2], sc[q][3]);
            const uint32_t r0 = pack2(sc[q][0] - bf_lo(h0), sc[q][1] - bf_hi(h0)), r1 = pack2(sc[q][2] - bf_lo(h1), sc[q][3] - bf_hi(h1));
            unsigned long long *p = (unsigned long long *)(pb + (((wave >> 1) * RT + q) * 2) * 64 + lane) + (wave & 1);
            p[0] = (unsigned long long)h0 | ((unsigned long long)h1 << 32);
            p[128] = (unsigned long long)r0 | ((unsigned long long)r1 << 32);
          } else {
            pb[(wave * RT + q) * 64 + lane] = (u32x4){__float_as_uint(sc[q][0]), __float_as_uint(sc[q][1]), __float_as_uint(sc[q][2]), __float_as_uint(sc[q][3])};
          }
        }
      }
      __syncthreads();
#pragma unroll
      for (int s = 0; s < SUB; s += B16 ? 2 : 1) {
        u32x4 p[RT][2], v[VBW];
#pragma unroll
        for (int q = 0; q < RT; q++) {
          if constexpr (B16) {
            p[q][0] = pb[(((s >> 1) * RT + q) * 2) * 64 + lane];
            p[q][1] = pb[(((s >> 1) * RT + q) * 2 + 1) * 64 + lane];
          } else {
            p[q][0] = pb[(s * RT + q) * 64 + lane];
          }
        }
#pragma unroll
        for (int j = 0; j < VBW; j++) v[j] = mx_value_operand(E(), kt, NK, s, wave + MK_WAVES * j, lane);  // (blocks behind the last are finite and never stored)
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int w = 0; w < (B16 ? 2 : 1); w++)
#pragma unroll
          for (int j = 0; j < VBW; j++)
#pragma unroll
            for (int q = 0; q < RT; q++) acc[q][j] = fx_mma_k(E(), v[j], p[q][w], acc[q][j]);
      }
    }
    MK_MARK(c, 1);
    // ---- sums of the wavefronts, then out (one chunk) or to the partial buffer
#pragma unroll
    for (int q = 0; q < RT; q++) {
      const float s = groups_sum(l[q]);
      if (lg == 0) ls[(wave * RT + q) * 16 + lr] = s;
    }
    __syncthreads();
#pragma unroll
    for (int q = 0; q < RT; q++) {
      const int r = q * 16 + lr;
      if (r < a.nrows) {
        float Lr = 0.f;
#pragma unroll
        for (int w = 0; w < MK_WAVES; w++) Lr += ls[(w * RT + q) * 16 + lr];
        if (a.C == 1) {
          const int Rw = a.r0 + r;
          E *o = (E *)st.out + (size_t)(a.t0 + Rw / H) * st.ld_out + (size_t)(Rw % H) * Rp;
          const float inv = 1.f / Lr;
#pragma unroll
          for (int j = 0; j < VBW; j++)
            if (wave + MK_WAVES * j < nvb) fx_stc_quad(o + (wave + MK_WAVES * j) * 16 + lg * 4, acc[q][j] * inv);
        } else {
          float *o = (float *)rt.attn_part + ((size_t)u * 16 * RT + r) * PST;
#pragma unroll
          for (int j = 0; j < VBW; j++)
            if (wave + MK_WAVES * j < nvb) mx_stc_quad(o + (wave + MK_WAVES * j) * 16 + lg * 4, acc[q][j]);
          if (wave == 0 && lg == 0) {
            stc_f32(o + Rp, m[q]);
            stc_f32(o + Rp + 1, Lr);
          }
        }
      }
    }
  }
  c.wrote_through = true;
}
// Rows of split requests.  Few chunks: a wavefront per (token, head), 256 values and eight chunks at a time.  Many chunks (few
// rows then): a wavefront per (token, head) and 64 values, a 16-lane row per chunk.
template <typename E>
__device__ __forceinline__ void stage_mx_latent_merge(CStage &st, Ctx &c, const MkRuntime &rt, int M) {
  barrier_wait(c);
  constexpr int KW = FxType<E>::KW;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lr = lane & 15, lg = lane >> 4;
  const int H = st.num_q_heads, Rp = (st.rank + KW - 1) / KW * KW, PST = Rp + 32, UR = 16 * st.v_tiles, TPOS = 16 * st.k_tiles;
  const MxLatentRows rw = mx_latent_rows(c, M, H, UR);
  const bool few = rw.cmax <= 8;
  const int bw = few ? 256 : 64, nb = (Rp + bw - 1) / bw;
  for (int ib = mx_wave_item(c, wave); ib < M * H * nb; ib += c.G * MK_WAVES) {
    const int i = ib / nb, blk = ib - i * nb, t = i / H, h = i - t * H, t0 = __builtin_amdgcn_readfirstlane(c.sh_tok[2 * MK_MAX_TOKENS + t]), Rw = (t - t0) * H + h;
    const int n = wave_bcast(rw.my_n, t0), item = wave_bcast(rw.tiles_incl, t0) - wave_bcast(rw.my_tiles, t0) + Rw / UR;
    const int C = mx_chunks((__builtin_amdgcn_readfirstlane(c.sh_tok[t0]) + n - 1) / TPOS + 1, rw.cmax);
    if (C == 1) continue;
    const float *p = (const float *)rt.attn_part + ((size_t)item * rw.cmax * UR + Rw % UR) * PST;
    const size_t step = (size_t)UR * PST;
    E *out = (E *)st.out + (size_t)t * st.ld_out + (size_t)h * Rp;
    // lane q holds chunk q's statistics
    const float mq = ldc_f32(p + min(lane, C - 1) * step + Rp), lq = ldc_f32(p + min(lane, C - 1) * step + Rp + 1);
    const int d = blk * bw + 4 * (few ? lane : lr), dc = min(d, Rp - 4);
    f32x4 x[8];
    auto load = [&](int q0) {
#pragma unroll
      for (int q = 0; q < 8; q++) x[q] = fx_ldc_quad(p + (size_t)min(few ? q0 + q : q0 + q * 4 + lg, C - 1) * step + dc);
    };
    load(0);
    float mm = lane < C ? mq : MK_FX_NEG;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mm = fmaxf(mm, __shfl_xor(mm, o));
    const float e = lane < C ? exp2f(mq - mm) : 0.f, inv = 1.f / wave_sum(lq * e);
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    for (int q0 = 0;;) {
#pragma unroll
      for (int q = 0; q < 8; q++) {
        const int at = few ? q0 + q : q0 + q * 4 + lg;
        const float f = __builtin_bit_cast(float, __builtin_amdgcn_ds_bpermute((at & 63) << 2, __builtin_bit_cast(int, e)));
        o += x[q] * (at < C ? f : 0.f);
      }
      q0 += few ? 8 : 32;
      if (q0 >= C) break;
      load(q0);
    }
    if (!few) {
#pragma unroll
      for (int y = 0; y < 4; y++) o[y] = groups_sum(o[y]);
    }
    if ((few || lg == 0) && d < Rp) fx_stc_quad(out + d, o * inv);
  }
  c.wrote_through = true;
}
template <typename E>
__device__ __forceinline__ void stage_mx_latent_attn(CStage &st, Ctx &c, const MkRuntime &rt, int M, char *smem) {
  // (the host picks st.nk, the operand rows of the instantiation, from this list)
  if constexpr (sizeof(E) == 2) {
    if (st.nk == 6) stage_mx_latent_attn_t<E, 6, 4, 2, 2>(st, c, rt, M, smem);
    else if (st.nk == 18) stage_mx_latent_attn_t<E, 18, 4, 8, 2>(st, c, rt, M, smem);
    else stage_mx_latent_attn_t<E, 20, 4, 8, 2>(st, c, rt, M, smem);
  } else {
    if (st.nk == 12) stage_mx_latent_attn_t<E, 12, 2, 2, 1>(st, c, rt, M, smem);
    else stage_mx_latent_attn_t<E, 40, 2, 8, 1>(st, c, rt, M, smem);
  }
}

// ----------------------------------------------------------------------------- generalised delta rule
// The columns of a head's state are independent of each other given the key-side vectors of a token.  A lane keeps NC columns x
// 4 NI channels in registers: lane l of a wavefront holds columns (l / 16) NC .. + NC - 1 of its wavefront's 4 NC and channels
// 64 i + 4 (l % 16) .. + 3, so the sums over channels stay inside a 16-lane row (four DPP additions).  State: 32-bit
// [slot][head][column][channel], sizes rounded up to 16; zero where a request begins.  Row sections of a head are padded with
// zeros to the same size Dp (D values count for the norm).  Decays come from the MX_DECAY form of the head linear.
//
// Iterations in which every request brings one token: a workgroup per (request, head), the next unit's state and rows in
// flight while one is computed.  Otherwise the rows of 16 tokens at a time are put in LDS by all wavefronts (the next 16 are in
// flight meanwhile) and every wavefront walks them; few units are dealt in slices of columns to several workgroups, which
// leave their unnormalised outputs to the MX_DELTA_OUT stage.
#define MX_TB 16
struct MxDeltaUnits {
  bool first;
  int my_n, rank_of, nreq;
};
__device__ __forceinline__ MxDeltaUnits mx_delta_units(const Ctx &c, int M) {
  const int lane = threadIdx.x & 63;
  MxDeltaUnits r;
  r.first = lane < M && c.sh_tok[2 * MK_MAX_TOKENS + lane] == lane;
  const unsigned long long fm = __ballot(r.first), later = lane < 63 ? fm >> (lane + 1) : 0ull;
  r.my_n = r.first ? (later ? (int)__ffsll(later) : M - lane) : 0;
  r.rank_of = __popcll(fm & ((1ull << lane) - 1ull));
  r.nreq = __popcll(fm);
  return r;
}
struct MxDeltaUnit {
  int h, t0, n, p0, col0;
  float *state;
};
// unit u of `slices` per (request, head), cols columns each
__device__ __forceinline__ MxDeltaUnit mx_delta_unit(CStage &st, const Ctx &c, const MkRuntime &rt, const MxDeltaUnits &us, int u, int slices, int cols, int Dp) {
  MxDeltaUnit a;
  const int uh = u / slices, H = st.num_q_heads, ri = uh / H;
  a.col0 = (u - uh * slices) * cols;
  a.h = uh - ri * H;
  a.t0 = (int)__ffsll(__ballot(us.first && us.rank_of == ri)) - 1;
  a.n = wave_bcast(us.my_n, a.t0);
  a.p0 = __builtin_amdgcn_readfirstlane(c.sh_tok[a.t0]);
  const int slot = __builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + a.t0]);
  a.state = (float *)st.k_cache + ((size_t)__builtin_amdgcn_readfirstlane(rt.state_ids[slot]) * H + a.h) * Dp * Dp;
  return a;
}
template <int NI, int NC>
__device__ __forceinline__ void mx_delta_load(f32x4 (&S)[NC][NI], const float *state, bool zero, int col, int lr, int Dp) {
#pragma unroll
  for (int j = 0; j < NC; j++)
#pragma unroll
    for (int i = 0; i < NI; i++) S[j][i] = __builtin_nontemporal_load((const f32x4 *)(state + (size_t)min(col + j, Dp - 1) * Dp + min(i * 64 + lr * 4, Dp - 4)));
#pragma unroll
  for (int j = 0; j < NC; j++)
#pragma unroll
    for (int i = 0; i < NI; i++)
      if (zero || col + j >= Dp || i * 64 + lr * 4 >= Dp) S[j][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
}
template <int NI, int NC>
__device__ __forceinline__ void mx_delta_store(const f32x4 (&S)[NC][NI], float *state, int col, int lr, int Dp) {
#pragma unroll
  for (int j = 0; j < NC; j++)
#pragma unroll
    for (int i = 0; i < NI; i++)
      if (col + j < Dp && i * 64 + lr * 4 < Dp) mx_stc_quad(state + (size_t)(col + j) * Dp + i * 64 + lr * 4, S[j][i]);
}
template <int NI> struct MxDeltaVec {
  f32x4 r[NI], k[NI], u[NI], au[NI], w[NI];
};
// one token: S <- diag(w) S - (a u)(u^T S) + k v^T, o = S^T r
template <int NI, int NC>
__device__ __forceinline__ void mx_delta_step(f32x4 (&S)[NC][NI], const MxDeltaVec<NI> &x, const float (&v)[NC], float (&o)[NC]) {
  float su[NC];
#pragma unroll
  for (int j = 0; j < NC; j++) {
    su[j] = 0.f;
#pragma unroll
    for (int i = 0; i < NI; i++)
#pragma unroll
      for (int e = 0; e < 4; e++) su[j] = fmaf(x.u[i][e], S[j][i][e], su[j]);
  }
#pragma unroll
  for (int j = 0; j < NC; j++) su[j] = group16_sum(su[j]);
#pragma unroll
  for (int j = 0; j < NC; j++) {
    o[j] = 0.f;
#pragma unroll
    for (int i = 0; i < NI; i++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        S[j][i][e] = fmaf(x.k[i][e], v[j], fmaf(-x.au[i][e], su[j], x.w[i][e] * S[j][i][e]));
        o[j] = fmaf(x.r[i][e], S[j][i][e], o[j]);
      }
  }
#pragma unroll
  for (int j = 0; j < NC; j++) o[j] = group16_sum(o[j]);
}
// every request brings one token
template <typename E, int NI, int NC>
__device__ __forceinline__ void stage_mx_delta_single(CStage &st, Ctx &c, const MkRuntime &rt, int M, char *smem) {
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int D = st.head_dim, Dp = (D + 15) / 16 * 16, H = st.num_q_heads, n_units = M * H, col = (wave * 4 + lg) * NC;
  const MxDeltaUnits us = mx_delta_units(c, M);
  const E *in = (const E *)st.in;
  const float *ab = (const float *)st.k_norm_w, *nw = (const float *)st.norm_w;
  float *red = (float *)smem;
  struct Raw {
    f32x4 r[NI], k[NI], a[NI], w[NI], ab[NI], v[NC / 4], g[NC / 4], nw[NC / 4];
  };
  auto load_raw = [&](const MxDeltaUnit &a, Raw &x) {
    const E *row = in + (size_t)a.t0 * st.ld_in + a.h * Dp;
    const float *wr = (const float *)st.in2 + (size_t)a.t0 * st.ld_in2 + a.h * Dp;
#pragma unroll
    for (int i = 0; i < NI; i++) {
      const int d = min(i * 64 + lr * 4, Dp - 4);
      x.r[i] = fx_ldc_quad(row + st.cols[0] + d);
      x.k[i] = fx_ldc_quad(row + st.cols[1] + d);
      x.a[i] = fx_ldc_quad(row + st.cols[4] + d);
      x.w[i] = fx_ldc_quad(wr + d);
      x.ab[i] = *(const f32x4 *)(ab + a.h * Dp + d);
    }
#pragma unroll
    for (int j = 0; j < NC / 4; j++) {
      const int d = min(col + 4 * j, Dp - 4);
      x.v[j] = fx_ldc_quad(row + st.cols[2] + d);
      x.g[j] = fx_ldc_quad(row + st.cols[3] + d);
      x.nw[j] = *(const f32x4 *)(nw + a.h * Dp + d);
    }
  };
  f32x4 S[NC][NI];
  const int u0 = mx_spread(c);
  MxDeltaUnit a{};
  // earlier iterations wrote the state: the first unit's is requested before the barrier is awaited
  const bool early = u0 < n_units && wave != 0;
  if (u0 < n_units) a = mx_delta_unit(st, c, rt, us, u0, 1, 0, Dp);
  if (early) mx_delta_load<NI, NC>(S, a.state, a.p0 == 0, col, lr, Dp);
  barrier_wait(c);
  Raw x;
  if (u0 < n_units) {
    if (!early) mx_delta_load<NI, NC>(S, a.state, a.p0 == 0, col, lr, Dp);
    load_raw(a, x);
  }
  int par = 0;
  for (int u = u0; u < n_units; u += c.G, par ^= 4) {
    MxDeltaUnit nx = a;
    f32x4 Sn[NC][NI];
    Raw xn;
    if (u + c.G < n_units) {
      nx = mx_delta_unit(st, c, rt, us, u + c.G, 1, 0, Dp);
      mx_delta_load<NI, NC>(Sn, nx.state, nx.p0 == 0, col, lr, Dp);
      load_raw(nx, xn);
    }
    MxDeltaVec<NI> y;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NI; i++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        if (i * 64 + lr * 4 >= Dp) x.r[i][e] = x.k[i][e] = 0.f;
        ss += x.k[i][e] * x.k[i][e];
      }
    const float inv = 1.f / sqrtf(group16_sum(ss) + 1e-6f);
#pragma unroll
    for (int i = 0; i < NI; i++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        y.r[i][e] = x.r[i][e];
        y.k[i][e] = x.k[i][e];
        y.u[i][e] = x.k[i][e] * inv;
        y.au[i][e] = mx_sigmoid(E(), x.a[i][e] + x.ab[i][e]) * y.u[i][e];
        y.w[i][e] = x.w[i][e];
      }
    float v[NC], o[NC];
#pragma unroll
    for (int j = 0; j < NC; j++) v[j] = col + j < Dp ? x.v[j / 4][j & 3] : 0.f;
    mx_delta_step<NI, NC>(S, y, v, o);
    mx_delta_store<NI, NC>(S, a.state, col, lr, Dp);
    float so = 0.f;
#pragma unroll
    for (int j = 0; j < NC; j++) so += o[j] * o[j];
    so = groups_sum(so);
    if (lane == 0) red[par + wave] = so;
    __syncthreads();
    const float rn = 1.f / sqrtf(((red[par] + red[par + 1]) + (red[par + 2] + red[par + 3])) / (float)D + st.eps);
    if (lr == 0) {
#pragma unroll
      for (int j = 0; j < NC / 4; j++) {
        f32x4 q;
#pragma unroll
        for (int e = 0; e < 4; e++) q[e] = (o[4 * j + e] * rn) * x.nw[j][e] * mx_sigmoid(E(), x.g[j][e]);
        if (col + 4 * j < Dp) fx_stc_quad((E *)st.out + (size_t)a.t0 * st.ld_out + a.h * Dp + col + 4 * j, q);
      }
    }
    a = nx;
    x = xn;
#pragma unroll
    for (int j = 0; j < NC; j++)
#pragma unroll
      for (int i = 0; i < NI; i++) S[j][i] = Sn[j][i];
  }
  c.wrote_through = true;
}

// some request brings several tokens: `slices` workgroups per (request, head), 16 NC columns each
template <typename E, int NI, int NC>
__device__ __forceinline__ void stage_mx_delta_multi(CStage &st, Ctx &c, const MkRuntime &rt, int M, int slices, char *smem) {
  constexpr int DPS = NI * 64 + 4, TW = MX_TB / MK_WAVES;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int D = st.head_dim, Dp = (D + 15) / 16 * 16, H = st.num_q_heads, cw = (wave * 4 + lg) * NC, d4 = min(4 * lane, Dp - 4);
  float *rv = (float *)smem, *kv = rv + MX_TB * DPS, *uv = kv + MX_TB * DPS, *av = uv + MX_TB * DPS, *wv = av + MX_TB * DPS, *vv = wv + MX_TB * DPS, *ov = vv + MX_TB * DPS;
  const MxDeltaUnits us = mx_delta_units(c, M);
  const int n_units = us.nreq * H * slices;
  const E *in = (const E *)st.in;
  const float *ab = (const float *)st.k_norm_w, *nw = (const float *)st.norm_w;
  f32x4 S[NC][NI];
  const int u0 = mx_spread(c);
  const bool early = u0 < n_units && wave != 0;
  if (early) {
    const MxDeltaUnit a = mx_delta_unit(st, c, rt, us, u0, slices, 16 * NC, Dp);
    mx_delta_load<NI, NC>(S, a.state, a.p0 == 0, a.col0 + cw, lr, Dp);
  }
  barrier_wait(c);
  for (int u = u0; u < n_units; u += c.G) {
    const MxDeltaUnit a = mx_delta_unit(st, c, rt, us, u, slices, 16 * NC, Dp);
    const int col = a.col0 + cw;
    if (!(u == u0 && early)) mx_delta_load<NI, NC>(S, a.state, a.p0 == 0, col, lr, Dp);
    // lane l of a wavefront takes channels 4 l .. + 3 of tokens wave, wave + 4, ... of the block
    f32x4 xr[TW], xk[TW], xv[TW], xa[TW], xw[TW];
    const f32x4 xab = *(const f32x4 *)(ab + a.h * Dp + d4), xnw = *(const f32x4 *)(nw + a.h * Dp + d4);
    auto load_rows = [&](int tb) {
#pragma unroll
      for (int j = 0; j < TW; j++) {
        const int t = a.t0 + min(tb + wave + j * MK_WAVES, a.n - 1);
        const E *row = in + (size_t)t * st.ld_in + a.h * Dp + d4;
        xr[j] = fx_ldc_quad(row + st.cols[0]);
        xk[j] = fx_ldc_quad(row + st.cols[1]);
        xv[j] = fx_ldc_quad(row + st.cols[2]);
        xa[j] = fx_ldc_quad(row + st.cols[4]);
        xw[j] = fx_ldc_quad((const float *)st.in2 + (size_t)t * st.ld_in2 + a.h * Dp + d4);
      }
    };
    load_rows(0);
    for (int tb = 0; tb < a.n; tb += MX_TB) {
      const int nt = min(MX_TB, a.n - tb);
      __syncthreads();  // LDS reuse
#pragma unroll
      for (int j = 0; j < TW; j++) {
        const bool real = 4 * lane < Dp;
        float ss = real ? xk[j][0] * xk[j][0] + xk[j][1] * xk[j][1] + xk[j][2] * xk[j][2] + xk[j][3] * xk[j][3] : 0.f;
        const float inv = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
        if (4 * lane < NI * 64) {
          f32x4 un, au;
#pragma unroll
          for (int e = 0; e < 4; e++) {
            if (!real) xr[j][e] = xk[j][e] = xv[j][e] = xw[j][e] = 0.f;
            un[e] = xk[j][e] * inv;
            au[e] = mx_sigmoid(E(), xa[j][e] + xab[e]) * un[e];
          }
          const int at = (wave + j * MK_WAVES) * DPS + 4 * lane;
          *(f32x4 *)(rv + at) = xr[j];
          *(f32x4 *)(kv + at) = xk[j];
          *(f32x4 *)(uv + at) = un;
          *(f32x4 *)(av + at) = au;
          *(f32x4 *)(wv + at) = xw[j];
          *(f32x4 *)(vv + at) = xv[j];
        }
      }
      load_rows(min(tb + MX_TB, a.n - 1));
      __syncthreads();
      auto load_vec = [&](int j, MxDeltaVec<NI> &y, float (&v)[NC]) {
#pragma unroll
        for (int i = 0; i < NI; i++) {
          const int at = j * DPS + i * 64 + lr * 4;
          y.r[i] = *(const f32x4 *)(rv + at);
          y.k[i] = *(const f32x4 *)(kv + at);
          y.u[i] = *(const f32x4 *)(uv + at);
          y.au[i] = *(const f32x4 *)(av + at);
          y.w[i] = *(const f32x4 *)(wv + at);
        }
#pragma unroll
        for (int q = 0; q < NC; q++) v[q] = vv[j * DPS + min(col + q, NI * 64 - 1)];
      };
      MxDeltaVec<NI> y;
      float v[NC];
      load_vec(0, y, v);
      for (int j = 0; j < nt; j++) {
        MxDeltaVec<NI> yn;
        float vn[NC], o[NC];
        load_vec(min(j + 1, nt - 1), yn, vn);
        mx_delta_step<NI, NC>(S, y, v, o);
        if (slices > 1) {
          float *row = (float *)st.out2 + (size_t)(a.t0 + tb + j) * st.ld_out2 + a.h * Dp;
          if (lr == 0) {
#pragma unroll
            for (int q = 0; q < NC; q++)
              if (col + q < Dp) stc_f32(row + col + q, o[q]);
          }
        } else if (lr == 0) {
#pragma unroll
          for (int q = 0; q < NC; q++) ov[j * DPS + min(col + q, NI * 64 - 1)] = o[q];
        }
        y = yn;
#pragma unroll
        for (int q = 0; q < NC; q++) v[q] = vn[q];
      }
      if (slices > 1) continue;
      __syncthreads();
      // ---- the head's outputs divided by their root mean square, weight, gate
      for (int j = wave; j < nt; j += MK_WAVES) {
        const size_t t = a.t0 + tb + j;
        const f32x4 g = fx_ldc_quad(in + t * st.ld_in + st.cols[3] + a.h * Dp + d4);
        const f32x4 o = *(const f32x4 *)(ov + j * DPS + d4);
        const float ss = 4 * lane < Dp ? o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3] : 0.f;
        const float rn = 1.f / sqrtf(wave_sum(ss) / (float)D + st.eps);
        f32x4 q;
#pragma unroll
        for (int e = 0; e < 4; e++) q[e] = (o[e] * rn) * xnw[e] * mx_sigmoid(E(), g[e]);
        if (4 * lane < Dp) fx_stc_quad((E *)st.out + t * st.ld_out + a.h * Dp + 4 * lane, q);
      }
    }
    mx_delta_store<NI, NC>(S, a.state, col, lr, Dp);
  }
  c.wrote_through = true;
}
// Head outputs of an iteration whose units were dealt in slices: a wavefront per (token, head).
template <typename E>
__device__ __forceinline__ void stage_mx_delta_out(CStage &st, Ctx &c, int M) {
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int D = st.head_dim, Dp = (D + 15) / 16 * 16, H = st.num_q_heads, d4 = min(4 * lane, Dp - 4);
  barrier_wait(c);
  for (int i = mx_wave_item(c, wave); i < M * H; i += c.G * MK_WAVES) {
    const int t = i / H, h = i - t * H;
    const f32x4 o = fx_ldc_quad((const float *)st.out2 + (size_t)t * st.ld_out2 + h * Dp + d4), g = fx_ldc_quad((const E *)st.in + (size_t)t * st.ld_in + st.cols[3] + h * Dp + d4),
                w = *(const f32x4 *)((const float *)st.norm_w + h * Dp + d4);
    const float ss = 4 * lane < Dp ? o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3] : 0.f;
    const float rn = 1.f / sqrtf(wave_sum(ss) / (float)D + st.eps);
    f32x4 q;
#pragma unroll
    for (int e = 0; e < 4; e++) q[e] = (o[e] * rn) * w[e] * mx_sigmoid(E(), g[e]);
    if (4 * lane < Dp) fx_stc_quad((E *)st.out + (size_t)t * st.ld_out + h * Dp + 4 * lane, q);
  }
  c.wrote_through = true;
}
template <typename E>
__device__ __forceinline__ void stage_mx_delta(CStage &st, Ctx &c, const MkRuntime &rt, int M, bool single, char *smem) {
  const int D = st.head_dim, Dp = (D + 15) / 16 * 16;
  c.mx_split = false;
  if (single && D <= 128) {
    if (D <= 64) stage_mx_delta_single<E, 1, 4>(st, c, rt, M, smem);
    else stage_mx_delta_single<E, 2, 8>(st, c, rt, M, smem);
    return;
  }
  // workgroups per (request, head) if every wavefront took as few columns as it can, and if they took all
  const int units = mx_delta_units(c, M).nreq * st.num_q_heads, fine = D <= 64 ? (Dp + 15) / 16 : (Dp + 31) / 32;
  const bool deal = units * fine <= c.G;
  if (D <= 64) {
    c.mx_split = deal && fine > 1;
    if (deal) stage_mx_delta_multi<E, 1, 1>(st, c, rt, M, fine, smem);
    else stage_mx_delta_multi<E, 1, 4>(st, c, rt, M, 1, smem);
  } else if (D <= 128) {
    c.mx_split = deal && fine > 1;
    if (deal) stage_mx_delta_multi<E, 2, 2>(st, c, rt, M, fine, smem);
    else stage_mx_delta_multi<E, 2, 8>(st, c, rt, M, 1, smem);
  } else {
    c.mx_split = true;
    stage_mx_delta_multi<E, 4, 2>(st, c, rt, M, fine, smem);
  }
}
