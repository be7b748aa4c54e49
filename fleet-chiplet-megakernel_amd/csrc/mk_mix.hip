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

// ----------------------------------------------------------------------------- residual sum + norm in parts
// v = x + alpha * f(y),  f(y) = y or y / sqrt(mean(y^2) + norm_eps) * y_norm_w;  out2 = v (32-bit);  out = the RMS norm of v in
// st.norm_groups equal parts times norm_w (norm_groups 0: v itself), rounded to E.  Rows are st.n long, st.k of them real (the
// rest is zero in every operand).  A workgroup per row.
template <typename E, int NS>
__device__ __forceinline__ void stage_mx_prenorm_t(CStage &st, Ctx &c, int M, char *smem) {
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
    for (int j = 0; j < NS; j++)
      if (j * MK_THREADS < n4) x[j] = fx_ldc_quad(xr + (size_t)t * st.ld_res + 4 * at(j));
  };
  if (ng) {
#pragma unroll
    for (int j = 0; j < NS; j++)
      if (j * MK_THREADS < n4) g[j] = w4[at(j)];
  }
  // the residual row was written at least one barrier earlier than y: requested before the barrier is awaited (not by the
  // wavefront that polls it)
  const bool pre = (st.flags & MK_F_RES_EARLY) && t0 < M && tid >= 64;
  if (pre) load_x(t0);
  barrier_wait(c);
  for (int t = t0; t < M; t += c.G) {
    if (!(pre && t == t0)) load_x(t);
    if (st.in) {
      f32x4 y[NS];
#pragma unroll
      for (int j = 0; j < NS; j++)
        if (j * MK_THREADS < n4) y[j] = fx_ldc_quad((const E *)st.in + (size_t)t * st.ld_in + 4 * at(j));
      float f = st.alpha;
      if (yw4) {
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < NS; j++)
          if (tid + j * MK_THREADS < n4) ss += y[j][0] * y[j][0] + y[j][1] * y[j][1] + y[j][2] * y[j][2] + y[j][3] * y[j][3];
        ss = block_sum(ss, red);
        const float r = 1.f / sqrtf(ss / (float)st.k + st.norm_eps);
#pragma unroll
        for (int j = 0; j < NS; j++)
          if (j * MK_THREADS < n4) y[j] = (y[j] * r) * yw4[at(j)];
      }
#pragma unroll
      for (int j = 0; j < NS; j++)
        if (j * MK_THREADS < n4) {
#pragma unroll
          for (int e = 0; e < 4; e++) x[j][e] = fmaf(f, y[j][e], x[j][e]);
        }
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
      }
    __syncthreads();
  }
  c.wrote_through = true;
}
template <typename E>
__device__ __forceinline__ void stage_mx_prenorm(CStage &st, Ctx &c, int M, char *smem) {
  if (st.n <= 4 * 4 * MK_THREADS) stage_mx_prenorm_t<E, 4>(st, c, M, smem);
  else stage_mx_prenorm_t<E, 12>(st, c, M, smem);
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
      const f32x4 y = fx_ldc_quad((const uint16_t *)st.y_in + 4 * i);
      ss += y[0] * y[0] + y[1] * y[1] + y[2] * y[2] + y[3] * y[3];
    }
    f = 1.f / sqrtf(block_sum(ss, red) / (float)st.k_real + st.norm_eps);
  }
  for (int i = tid; i < k4; i += MK_THREADS) {
    f32x4 v = fx_ldc_quad((const float *)st.res + 4 * i);
    if (st.y_in) {
      f32x4 y = fx_ldc_quad((const uint16_t *)st.y_in + 4 * i);
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
  const bool early = st.flags & MK_F_RES_EARLY;
  if (early) load_x();
  if (c.pending && lane == 0) barrier_poll(c);
  if (!early) load_x();
  if (st.y_in) {
    u32x4 y[KL];
#pragma unroll
    for (int kc = 0; kc < KL; kc++) y[kc] = ldc_16B((const u32x4 *)st.y_in + kc * 64 + lane);
    auto ye = [&](int kc, int h, int e) { return (e & 1) ? bf_hi(y[kc][h * 2 + (e >> 1)]) : bf_lo(y[kc][h * 2 + (e >> 1)]); };
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
      o[e] = g / (1.f + expf(-beta * g)) * (u + bias);
    }
    fx_stc_quad((E *)st.glu_out + (size_t)t * st.ld_glu + d, o);
  }
}

// ----------------------------------------------------------------------------- latent rows
// One wavefront: row of n values (n4 quads are readable, those behind n are zero) / rms * w; put(quad index, values).
template <typename E, typename Put>
__device__ __forceinline__ void mx_norm_row(const E *src, const float *w, int n, float eps, int lane, Put put) {
  constexpr int NQ = MK_MX_MAX_NORM_ROW / 256;
  const int n4 = (n + 3) / 4;
  f32x4 v[NQ];
#pragma unroll
  for (int j = 0; j < NQ; j++)
    if (j * 64 < n4) v[j] = fx_ldc_quad(src + 4 * min(j * 64 + lane, n4 - 1));
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NQ; j++)
    if (j * 64 + lane < n4) ss += v[j][0] * v[j][0] + v[j][1] * v[j][1] + v[j][2] * v[j][2] + v[j][3] * v[j][3];
  const float r = 1.f / sqrtf(wave_sum(ss) / (float)n + eps);
#pragma unroll
  for (int j = 0; j < NQ; j++)
    if (j * 64 + lane < n4) {
      const f32x4 g = ((const f32x4 *)w)[j * 64 + lane];
      put(j * 64 + lane, (v[j] * r) * g);
    }
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
  const int per = st.k_cache ? 2 : 1, total = M * per, w0 = mx_spread(c);
  for (int i = w0 + wave * c.G; i < total; i += c.G * MK_WAVES) {
    const int t = i / per;
    const E *row = (const E *)st.in + (size_t)t * st.ld_in;
    if (i - t * per == 0) {
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
// are [head][n / 16][k / KW][64 lanes][EPC]: lane l holds row l % 16, k (l / 16) * EPC .. .  A wavefront per 16-row tile; few
// tiles with long rows: a workgroup per tile, its wavefronts split K.  MK_F_GELU_TABLE: out = gelu(sum) * table[id(t)][n].
template <typename E, int MT, bool SPLIT>
__device__ __forceinline__ void stage_mx_head_linear_t(CStage &st, Ctx &c, int M, char *smem) {
  constexpr int EPC = FxType<E>::EPC, KW = FxType<E>::KW, KB = MT == 4 ? 4 : 8;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int N = st.n, nks = st.k / KW, nt = (N + 15) / 16, tiles = st.groups * nt;
  const int kq = SPLIT ? (nks + MK_WAVES - 1) / MK_WAVES : nks;
  const int kb = SPLIT ? min(nks, wave * kq) : 0, ke = SPLIT ? min(nks, kb + kq) : nks;
  const u32x4 *W = (const u32x4 *)st.w.seg[0];
  const int i0 = SPLIT ? mx_spread(c) : mx_spread(c) + wave * c.G, di = SPLIT ? c.G : c.G * MK_WAVES;
  f32x4 *red = (f32x4 *)smem;
  u32x4 a[KB];
  auto load_w = [&](int i, int k0) {
#pragma unroll
    for (int j = 0; j < KB; j++) a[j] = ldg_stream(W + ((size_t)i * nks + min(k0 + j, nks - 1)) * 64 + lane);
  };
  // weights do not depend on the previous stage: the first tile's are requested before its barrier completes
  const bool early = i0 < tiles && wave != 0;
  if (early) load_w(i0, kb);
  if (tid == 0) __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
  barrier_wait(c);
  for (int i = i0; i < tiles; i += di) {
    const int h = i / nt, n0 = (i - h * nt) * 16 + lg * 4;
    const E *xr[MT];
#pragma unroll
    for (int m = 0; m < MT; m++) xr[m] = (const E *)st.in + (size_t)min(m * 16 + lr, M - 1) * st.ld_in + (size_t)h * st.ld_in_slot + lg * EPC;
    f32x4 acc[MT];
#pragma unroll
    for (int m = 0; m < MT; m++) acc[m] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int k0 = kb; k0 < ke; k0 += KB) {
      if (!(early && i == i0 && k0 == kb)) load_w(i, k0);
#pragma unroll
      for (int j = 0; j < KB; j++) {
        const int ks = min(k0 + j, nks - 1);
        u32x4 b[MT];
#pragma unroll
        for (int m = 0; m < MT; m++) b[m] = *(const u32x4 *)(xr[m] + (size_t)ks * KW);
        if (k0 + j < ke) {
#pragma unroll
          for (int m = 0; m < MT; m++) acc[m] = fx_mma_k(E(), a[j], b[m], acc[m]);
        }
      }
    }
    if constexpr (SPLIT) {
      __syncthreads();
#pragma unroll
      for (int m = 0; m < MT; m++) red[(wave * MT + m) * 64 + lane] = acc[m];
      __syncthreads();
    }
#pragma unroll
    for (int m = 0; m < MT; m++) {
      if (SPLIT && m % MK_WAVES != wave) continue;
      f32x4 v = acc[m];
      if constexpr (SPLIT) {
        v = red[m * 64 + lane];
#pragma unroll
        for (int w = 1; w < MK_WAVES; w++) v += red[(w * MT + m) * 64 + lane];
      }
      const int t = m * 16 + lr;
      if (t >= M) continue;
      float r[4] = {v[0], v[1], v[2], v[3]};
      if (st.flags & MK_F_GELU_TABLE) {
        const long long id = (long long)ldc_u64((const long long *)st.aux0 + t);
        const E *e = (const E *)st.aux1 + (size_t)(id < 0 ? 0 : id) * st.ld_res;
#pragma unroll
        for (int q = 0; q < 4; q++) {
          const float z = r[q], th = tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z));
          r[q] = (id < 0 || n0 + q >= N) ? 0.f : 0.5f * z * (1.f + th) * fx_val(e[n0 + q]);
        }
      }
      fx_stc4((E *)st.out + (size_t)t * st.ld_out + (size_t)h * st.ld_out_slot, n0, N, r);
    }
  }
  c.wrote_through = true;
}
template <typename E, int MAXM>
__device__ __forceinline__ void stage_mx_head_linear(CStage &st, Ctx &c, int M, char *smem) {
  const bool split = st.groups * ((st.n + 15) / 16) <= c.G && st.k / FxType<E>::KW >= 8;
  if (split) {
    if (MAXM == 1 || M <= 16) stage_mx_head_linear_t<E, 1, true>(st, c, M, smem);
    else stage_mx_head_linear_t<E, 4, true>(st, c, M, smem);
  } else {
    if (MAXM == 1 || M <= 16) stage_mx_head_linear_t<E, 1, false>(st, c, M, smem);
    else stage_mx_head_linear_t<E, 4, false>(st, c, M, smem);
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
  r.cmax = max(1, min(c.G / r.total, MK_ATTN_MAX_CHUNKS));
  return r;
}
// Chunks of a unit with NT tiles.
__device__ __forceinline__ int mx_chunks(int NT, int cmax) { return NT <= 2 ? 1 : min(cmax, NT <= 16 ? NT : max(16, (NT + 1) / 2)); }

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

template <typename E, int KC, int VBW, int RT>
__device__ __forceinline__ void stage_mx_latent_attn_t(CStage &st, Ctx &c, const MkRuntime &rt, int M, char *smem) {
  using X = FxType<E>;
  constexpr int EPC = X::EPC, KW = X::KW, B16 = sizeof(E) == 2;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int H = st.num_q_heads, R = st.rank, rot = st.rot_dims, half = rot / 2;
  const int nrc = (R + KW - 1) / KW, nkc = nrc + (rot + KW - 1) / KW, nvb = nrc * KW / 16, Rp = nrc * KW, PST = Rp + 32;
  const int SUB = st.k_tiles, TPOS = 16 * SUB, parts = MK_WAVES / SUB, ps = rt.page_size;
  const int my_sub = wave & (SUB - 1), my_part = wave / SUB;
  const MkLatentLds L = mk_latent_lds(sizeof(E), RT, nkc, SUB, 0);
  u32x4 *qs = (u32x4 *)smem;
  char *kt = smem + L.kt;
  u32x4 *pb = (u32x4 *)(smem + L.pb);
  float *mx = (float *)(smem + L.mx), *ls = mx + 4 * RT * 16;
  int *spg = (int *)(smem + L.pages);
  const u32x4 *kc = (const u32x4 *)st.k_cache;
  const MxLatentRows rw = mx_latent_rows(c, M, H, 16 * RT);
  const int cmax = rw.cmax, n_units = rw.total * cmax;
  c.mx_split = false;
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
    for (int j = 0; j < KC; j++)
      if (j * parts < nkc) kv[j] = p[min(j * parts + my_part, nkc - 1) * 64];
  };
  auto store_tile = [&](int tile, int newest) {
    const bool hidden = tile * TPOS + my_sub * 16 + lr > newest;  // rows behind the newest position belong to nobody
#pragma unroll
    for (int j = 0; j < KC; j++) {
      const int ch = j * parts + my_part;
      if (ch < nkc) ((u32x4 *)kt)[(my_sub * nkc + ch) * 64 + lane] = hidden ? (u32x4){0u, 0u, 0u, 0u} : kv[j];
    }
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
    const int pg_lo = a.tb * TPOS / ps, npg = a.tb < a.te ? (a.te * TPOS - 1) / ps - pg_lo + 1 : 0;
    for (int i = tid; i < npg; i += MK_THREADS) spg[i] = rt.kv_indices[a.pages + min(pg_lo + i, a.p / ps)];
    // ---- query rows in operand order, the rotated part on the way
    for (int i = tid; i < RT * nkc * 64; i += MK_THREADS) {
      const int rc = i >> 6, rtile = rc / nkc, ch = rc - rtile * nkc, r = rtile * 16 + (i & 15), g = (i & 63) >> 4, Rw = a.r0 + r;
      u32x4 v = {0u, 0u, 0u, 0u};
      if (r < a.nrows) {
        const int t = a.t0 + Rw / H, h = Rw % H;
        if (ch < nrc) {
          v = ldc_16B((const u32x4 *)((const E *)st.q_ws + (size_t)t * st.ld_qws + (size_t)h * Rp + ch * KW + g * EPC));
        } else {
          const E *q = (const E *)st.in + (size_t)t * st.ld_in + (size_t)h * st.ld_in_slot + st.cols[0];
          const int pos = c.sh_tok[t];
          const float *ct = (const float *)st.cos_tab + (size_t)pos * st.ld_cos, *sn = (const float *)st.sin_tab + (size_t)pos * st.ld_cos;
          float f[EPC];
#pragma unroll
          for (int e = 0; e < EPC; e++) {
            const int d = (ch - nrc) * KW + g * EPC + e;
            f[e] = 0.f;
            if (d < rot) {
              const int k = d < half ? d : d - half;
              const float x = fx_ldc(q + d), y = fx_ldc(q + (d < half ? d + half : k));
              f[e] = d < half ? x * ct[k] - y * sn[k] : x * ct[k] + y * sn[k];
            }
          }
          if constexpr (B16) {
#pragma unroll
            for (int w = 0; w < 4; w++) v[w] = pack2(f[(2 * w) % EPC], f[(2 * w + 1) % EPC]);
          } else {
#pragma unroll
            for (int w = 0; w < 4; w++) v[w] = __float_as_uint(f[w % EPC]);
          }
        }
      }
      qs[i] = v;
    }
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
      if (wave < SUB) {
        f32x4 S[RT];
#pragma unroll
        for (int q = 0; q < RT; q++) S[q] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
        for (int ch = 0; ch < nkc; ch++) {
          const u32x4 k = ((const u32x4 *)kt)[(wave * nkc + ch) * 64 + lane];
#pragma unroll
          for (int q = 0; q < RT; q++) S[q] = fx_mma_k(E(), k, qs[(q * nkc + ch) * 64 + lane], S[q]);
        }
#pragma unroll
        for (int q = 0; q < RT; q++) {
          float tm = MK_FX_NEG;
#pragma unroll
          for (int i = 0; i < 4; i++) {
            sc[q][i] = tile * TPOS + wave * 16 + lg * 4 + i <= plim[q] ? S[q][i] * sc1 : MK_FX_NEG;
            tm = fmaxf(tm, sc[q][i]);
          }
          tm = groups_max(tm);
          if (lg == 0) mx[(wave * RT + q) * 16 + lr] = tm;
        }
      }
      __syncthreads();
#pragma unroll
      for (int q = 0; q < RT; q++) {
        float nm = m[q];
        for (int s = 0; s < SUB; s++) nm = fmaxf(nm, mx[(s * RT + q) * 16 + lr]);
        if (__any(nm > m[q])) {
          const float corr = fx_exp2(E(), m[q] - nm);
          m[q] = nm;
          l[q] *= corr;
#pragma unroll
          for (int b = 0; b < VBW; b++) acc[q][b] *= corr;
        }
        if (wave < SUB) {
#pragma unroll
          for (int i = 0; i < 4; i++) {
            sc[q][i] = sc[q][i] > 0.5f * MK_FX_NEG ? fx_exp2(E(), sc[q][i] - nm) : 0.f;
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
      for (int s = 0; s < SUB; s += B16 ? 2 : 1) {
#pragma unroll
        for (int j = 0; j < VBW; j++) {
          const int b = wave + MK_WAVES * j;
          if (b < nvb) {
            const u32x4 v = mx_value_operand(E(), kt, nkc, s, b, lane);
#pragma unroll
            for (int q = 0; q < RT; q++) {
              if (q * 16 < a.nrows) {
                if constexpr (B16) {
                  const u32x4 *p = pb + (((s >> 1) * RT + q) * 2) * 64 + lane;
                  acc[q][j] = fx_mma_k(E(), v, p[0], acc[q][j]);
                  acc[q][j] = fx_mma_k(E(), v, p[64], acc[q][j]);
                } else {
                  acc[q][j] = fx_mma_k(E(), v, pb[(s * RT + q) * 64 + lane], acc[q][j]);
                }
              }
            }
          }
        }
      }
    }
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
            if (wave + MK_WAVES * j < nvb) fx_stc_quad(o + (wave + MK_WAVES * j) * 16 + lg * 4, acc[q][j]);
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
// Rows of split requests: a wavefront per (token, head).
template <typename E>
__device__ __forceinline__ void stage_mx_latent_merge(CStage &st, Ctx &c, const MkRuntime &rt, int M) {
  barrier_wait(c);
  constexpr int KW = FxType<E>::KW;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int H = st.num_q_heads, Rp = (st.rank + KW - 1) / KW * KW, PST = Rp + 32, UR = 16 * st.v_tiles, TPOS = 16 * st.k_tiles;
  const MxLatentRows rw = mx_latent_rows(c, M, H, UR);
  for (int i = mx_spread(c) + wave * c.G; i < M * H; i += c.G * MK_WAVES) {
    const int t = i / H, h = i - t * H, t0 = __builtin_amdgcn_readfirstlane(c.sh_tok[2 * MK_MAX_TOKENS + t]), Rw = (t - t0) * H + h;
    const int n = wave_bcast(rw.my_n, t0), item = wave_bcast(rw.tiles_incl, t0) - wave_bcast(rw.my_tiles, t0) + Rw / UR;
    const int C = mx_chunks((__builtin_amdgcn_readfirstlane(c.sh_tok[t0]) + n - 1) / TPOS + 1, rw.cmax);
    if (C == 1) continue;
    const float *p = (const float *)rt.attn_part + ((size_t)item * rw.cmax * UR + Rw % UR) * PST;
    const size_t step = (size_t)UR * PST;
    // lane q holds chunk q's statistics
    const float mq = lane < C ? ldc_f32(p + lane * step + Rp) : MK_FX_NEG, lq = lane < C ? ldc_f32(p + lane * step + Rp + 1) : 0.f;
    float mm = mq;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) mm = fmaxf(mm, __shfl_xor(mm, o));
    const float e = lane < C ? exp2f(mq - mm) : 0.f, inv = 1.f / wave_sum(lq * e);
    E *out = (E *)st.out + (size_t)t * st.ld_out + (size_t)h * Rp;
    for (int d = 4 * lane; d < (Rp + 255) / 256 * 256; d += 256) {
      f32x4 o = {0.f, 0.f, 0.f, 0.f};
      for (int q0 = 0; q0 < C; q0 += 8) {
        f32x4 x[8];
#pragma unroll
        for (int q = 0; q < 8; q++) x[q] = fx_ldc_quad(p + min(q0 + q, C - 1) * step + min(d, Rp - 4));
#pragma unroll
        for (int q = 0; q < 8; q++) {
          const float f = lane_f32(e, min(q0 + q, C - 1));
          if (q0 + q < C) o += x[q] * f;
        }
      }
      if (d < Rp) fx_stc_quad(out + d, o * inv);
    }
  }
  c.wrote_through = true;
}
template <typename E>
__device__ __forceinline__ void stage_mx_latent_attn(CStage &st, Ctx &c, const MkRuntime &rt, int M, char *smem) {
  if constexpr (sizeof(E) == 2) {
    if (st.rank <= 128 && st.rot_dims <= 64) stage_mx_latent_attn_t<E, 6, 2, 2>(st, c, rt, M, smem);
    else stage_mx_latent_attn_t<E, 20, 8, 2>(st, c, rt, M, smem);
  } else {
    stage_mx_latent_attn_t<E, 20, 8, 1>(st, c, rt, M, smem);
  }
}

// ----------------------------------------------------------------------------- generalised delta rule
// Unit = (request, head), a workgroup each; a token block of 16 rows at a time.  The columns of the state are independent of
// each other given the block's key-side vectors, so a wavefront keeps 16-column blocks of it in registers (lane l: column
// l % 16, channels 16 i + 4 (l / 16) .. + 3) and walks the tokens; the two sums over channels cross lanes with two swaps.
// The key-side vectors (unit key, removal, decay) are formed first, the decay's low-rank product on the matrix cores.
// State: [slot][head][column block][i][64 lanes] f32x4, 32-bit; zero where a request begins.
#define MX_TB 16
template <typename E, int DQ, int NB>
__device__ __forceinline__ void stage_mx_delta_t(CStage &st, Ctx &c, const MkRuntime &rt, int M, char *smem) {
  constexpr int EPC = FxType<E>::EPC, KW = FxType<E>::KW, B16 = sizeof(E) == 2, DP = DQ * 16, DPS = DP + 4;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int D = st.head_dim, H = st.num_q_heads, nd = (D + 15) / 16, nks = st.rank / KW, passes = (nd + MK_WAVES * NB - 1) / (MK_WAVES * NB);
  float *rv = (float *)smem, *kv = rv + MX_TB * DPS, *uv = kv + MX_TB * DPS, *av = uv + MX_TB * DPS, *wv = av + MX_TB * DPS, *vv = wv + MX_TB * DPS;
  u32x4 *tw = (u32x4 *)(vv + MX_TB * DPS);  // [rank / KW][value, remainder][64] operands of tanh(low-rank projection)
  const bool first = lane < M && c.sh_tok[2 * MK_MAX_TOKENS + lane] == lane;
  const unsigned long long fm = __ballot(first), later = lane < 63 ? fm >> (lane + 1) : 0ull;
  const int my_n = first ? (later ? (int)__ffsll(later) : M - lane) : 0;
  const int rank_of = __popcll(fm & ((1ull << lane) - 1ull)), n_units = __popcll(fm) * H;
  struct Unit {
    int h, t0, n, p0;
    f32x4 *state;
  };
  auto decode = [&](int u) {
    Unit a;
    const int ri = u / H;
    a.h = u - ri * H;
    a.t0 = (int)__ffsll(__ballot(first && rank_of == ri)) - 1;
    a.n = wave_bcast(my_n, a.t0);
    a.p0 = __builtin_amdgcn_readfirstlane(c.sh_tok[a.t0]);
    const int slot = __builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + a.t0]);
    a.state = (f32x4 *)st.k_cache + ((size_t)rt.state_ids[slot] * H + a.h) * nd * nd * 64 + lane;
    return a;
  };
  f32x4 S[NB][DQ];
  auto load_state = [&](const Unit &a, int pass, bool zero) {
#pragma unroll
    for (int b = 0; b < NB; b++) {
      const int cb = (pass * NB + b) * MK_WAVES + wave;
#pragma unroll
      for (int i = 0; i < DQ; i++) {
        S[b][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
        if (!zero && i < nd && cb < nd) S[b][i] = fx_ldc_quad((const float *)(a.state + (size_t)(cb * nd + i) * 64));
      }
    }
  };
  auto store_state = [&](const Unit &a, int pass) {
#pragma unroll
    for (int b = 0; b < NB; b++) {
      const int cb = (pass * NB + b) * MK_WAVES + wave;
#pragma unroll
      for (int i = 0; i < DQ; i++)
        if (i < nd && cb < nd) fx_stc_quad((float *)(a.state + (size_t)(cb * nd + i) * 64), S[b][i]);
    }
  };
  const int u0 = mx_spread(c);
  // earlier iterations wrote the state: the first unit's is requested before the barrier is awaited
  const bool early = passes == 1 && u0 < n_units && wave != 0;
  if (early) {
    const Unit a = decode(u0);
    load_state(a, 0, a.p0 == 0);
  }
  barrier_wait(c);
  const E *in = (const E *)st.in;
  const float *w0 = (const float *)st.q_norm_w, *ab = (const float *)st.k_norm_w, *nw = (const float *)st.norm_w;
  for (int u = u0; u < n_units; u += c.G) {
    const Unit a = decode(u);
    if (passes == 1 && !(u == u0 && early)) load_state(a, 0, a.p0 == 0);
    for (int tb = 0; tb < a.n; tb += MX_TB) {
      const int nt = min(MX_TB, a.n - tb);
      __syncthreads();  // LDS reuse
      // ---- rows: r, k, v as they are, u = k / |k|, a u
      for (int j = wave; j < nt; j += MK_WAVES) {
        const E *row = in + (size_t)(a.t0 + tb + j) * st.ld_in + a.h * D;
        float xr[DP / 64], xk[DP / 64], xv[DP / 64], xa[DP / 64], ss = 0.f;
#pragma unroll
        for (int i = 0; i < DP / 64; i++) {
          const int d = min(i * 64 + lane, D - 1);
          xr[i] = fx_ldc(row + st.cols[0] + d);
          xk[i] = fx_ldc(row + st.cols[1] + d);
          xv[i] = fx_ldc(row + st.cols[2] + d);
          xa[i] = fx_ldc(row + st.cols[4] + d);
        }
#pragma unroll
        for (int i = 0; i < DP / 64; i++) {
          if (i * 64 + lane >= D) xr[i] = xk[i] = xv[i] = 0.f;
          ss += xk[i] * xk[i];
        }
        const float inv = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
#pragma unroll
        for (int i = 0; i < DP / 64; i++) {
          const int d = i * 64 + lane, at = j * DPS + d;
          const float un = xk[i] * inv, rem = d < D ? 1.f / (1.f + expf(-(xa[i] + ab[a.h * D + min(d, D - 1)]))) : 0.f;
          rv[at] = xr[i];
          kv[at] = xk[i];
          vv[at] = xv[i];
          uv[at] = un;
          av[at] = rem * un;
        }
      }
      for (int i = tid; i < nks * 64; i += MK_THREADS) {
        const int ks = i >> 6, t = i & 15, k = ks * KW + ((i & 63) >> 4) * EPC;
        const E *row = in + (size_t)(a.t0 + tb + min(t, nt - 1)) * st.ld_in + st.cols[5] + k;
        float f[EPC];
#pragma unroll
        for (int e = 0; e < EPC; e += 4) {
          const f32x4 q = fx_ldc_quad(row + e);
#pragma unroll
          for (int y = 0; y < 4; y++) f[e + y] = tanhf(q[y]);
        }
        u32x4 hi, lo;
#pragma unroll
        for (int w = 0; w < 4; w++) {
          if constexpr (B16) {
            const float x0 = f[(2 * w) % EPC], x1 = f[(2 * w + 1) % EPC];
            hi[w] = pack2(x0, x1);
            lo[w] = pack2(x0 - bf_lo(hi[w]), x1 - bf_hi(hi[w]));
          } else {
            hi[w] = __float_as_uint(f[w % EPC]);
            lo[w] = 0u;
          }
        }
        tw[(ks * 2) * 64 + (i & 63)] = hi;
        if constexpr (B16) tw[(ks * 2 + 1) * 64 + (i & 63)] = lo;
      }
      __syncthreads();
      // ---- decays of 16 channels x 16 tokens at a time
      for (int ct = wave; ct < DQ; ct += MK_WAVES) {
        f32x4 z = {0.f, 0.f, 0.f, 0.f};
        if (ct < nd) {
          const u32x4 *wt = (const u32x4 *)st.w.seg[0] + ((size_t)a.h * nd + ct) * nks * 64 + lane;
          for (int ks = 0; ks < nks; ks++) {
            const u32x4 w = wt[ks * 64];
            z = fx_mma_k(E(), w, tw[(ks * 2) * 64 + lane], z);
            if constexpr (B16) z = fx_mma_k(E(), w, tw[(ks * 2 + 1) * 64 + lane], z);
          }
        }
        f32x4 w;
#pragma unroll
        for (int i = 0; i < 4; i++) {
          const int d = ct * 16 + lg * 4 + i;
          w[i] = d < D ? expf(-0.6065306597126334f / (1.f + expf(-(z[i] + w0[a.h * D + min(d, D - 1)])))) : 0.f;
        }
        *(f32x4 *)(wv + lr * DPS + ct * 16 + lg * 4) = w;
      }
      __syncthreads();
      // ---- tokens
      for (int pass = 0; pass < passes; pass++) {
        if (passes > 1) load_state(a, pass, a.p0 == 0 && tb == 0);
        for (int j = 0; j < nt; j++) {
          const size_t o4 = (size_t)(j * DPS + lg * 4);
          float su[NB], so[NB], v[NB];
#pragma unroll
          for (int b = 0; b < NB; b++) {
            su[b] = so[b] = 0.f;
            v[b] = vv[j * DPS + min(((pass * NB + b) * MK_WAVES + wave) * 16, DP - 16) + lr];
          }
#pragma unroll
          for (int i = 0; i < DQ; i++) {
            const f32x4 q = *(const f32x4 *)(uv + o4 + i * 16);
#pragma unroll
            for (int b = 0; b < NB; b++)
#pragma unroll
              for (int e = 0; e < 4; e++) su[b] = fmaf(q[e], S[b][i][e], su[b]);
          }
#pragma unroll
          for (int b = 0; b < NB; b++) su[b] = groups_sum(su[b]);
#pragma unroll
          for (int i = 0; i < DQ; i++) {
            const f32x4 w = *(const f32x4 *)(wv + o4 + i * 16), q = *(const f32x4 *)(av + o4 + i * 16), k = *(const f32x4 *)(kv + o4 + i * 16),
                        r = *(const f32x4 *)(rv + o4 + i * 16);
#pragma unroll
            for (int b = 0; b < NB; b++)
#pragma unroll
              for (int e = 0; e < 4; e++) {
                S[b][i][e] = fmaf(k[e], v[b], fmaf(-q[e], su[b], w[e] * S[b][i][e]));
                so[b] = fmaf(r[e], S[b][i][e], so[b]);
              }
          }
#pragma unroll
          for (int b = 0; b < NB; b++) {
            so[b] = groups_sum(so[b]);
            const int cb = (pass * NB + b) * MK_WAVES + wave;
            if (lg == 0 && cb < nd) vv[j * DPS + cb * 16 + lr] = so[b];  // (v of these columns is this wavefront's own)
          }
        }
        if (passes > 1) store_state(a, pass);
      }
      __syncthreads();
      // ---- each head's output divided by its root mean square, weight, gate
      for (int j = wave; j < nt; j += MK_WAVES) {
        const size_t t = a.t0 + tb + j;
        float o[DP / 64], g[DP / 64], ss = 0.f;
#pragma unroll
        for (int i = 0; i < DP / 64; i++) {
          const int d = i * 64 + lane;
          g[i] = fx_ldc(in + t * st.ld_in + st.cols[3] + a.h * D + min(d, D - 1));
          o[i] = d < D ? vv[j * DPS + d] : 0.f;
          ss += o[i] * o[i];
        }
        const float inv = 1.f / sqrtf(wave_sum(ss) / (float)D + st.eps);
#pragma unroll
        for (int i = 0; i < DP / 64; i++) {
          const int d = i * 64 + lane;
          if (d < D) fx_stc((E *)st.out + t * st.ld_out + a.h * D + d, fx_round<E>((o[i] * inv) * nw[a.h * D + d] / (1.f + expf(-g[i]))));
        }
      }
    }
    if (passes == 1) store_state(a, 0);
  }
  mx_glu<E>(st, c, M);
  c.wrote_through = true;
}
template <typename E>
__device__ __forceinline__ void stage_mx_delta(CStage &st, Ctx &c, const MkRuntime &rt, int M, char *smem) {
  if (st.head_dim <= 64) stage_mx_delta_t<E, 4, 1>(st, c, rt, M, smem);
  else if (st.head_dim <= 128) stage_mx_delta_t<E, 8, 2>(st, c, rt, M, smem);
  else stage_mx_delta_t<E, 16, 1>(st, c, rt, M, smem);
}
