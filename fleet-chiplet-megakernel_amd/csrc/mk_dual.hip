// Convolutions that keep a ring of rows and the state-space recurrence with one decay per head (part of the persistent kernel,
// included by mk_kernel.hip behind mk_hybrid.hip, whose conventions it keeps: sizes and constants are descriptor fields, E is the
// type of activations and weights, everything named in 32 bits is 32-bit in both builds).
//   * stage_du_conv   causal convolution per channel: with silu and a bias, or added to its own input; step sizes and decays beside it;
//   * stage_du_scan   S' = a S + dt B x^T, y = (S'^T C + D x) silu(z) per head, state per request.
// (Two sub-layers that join the residual stream together, and the convolution of single tokens, are in the norm stage, stage_mx_prenorm;
// chunks, score factors and norms over whole rows of heads in stage_fx_attn; groups of experts and the clamped activation in mk_hybrid.hip.)

// ----------------------------------------------------------------------------- convolution
// out[t, c] = act(b[c] + sum_j w[j][c] x[t - (taps - 1) + j, c]), x = in[t, cols[0] + c], st.n channels (a multiple of 4); MK_F_SILU: act
// is silu, MK_F_IDENTITY: x[t, c] itself is added.  A request's ring [taps][n] holds the input of position p in row p % taps.  Whoever
// takes a request's first token takes the taps - 1 first ones, which read the ring, and then puts the last inputs there; the other
// tokens of a portion are independent.  Steps: dt[t, h] = softplus(in[t, cols[1] + h] + step_bias[h]) and a[t, h] = 2^(rate[h] dt) go to
// 32-bit rows (out2: steps, from column cols[2] on decays).
template <typename E>
__device__ __forceinline__ void stage_du_conv(CStage &st, Ctx &c, int M) {
  const int n = st.n, n4 = n / 4, taps = st.taps, per = (n4 + MK_THREADS - 1) / MK_THREADS, lane = threadIdx.x & 63;
  const int H = st.step_bias ? st.num_q_heads : 0, hper = (H + MK_THREADS - 1) / MK_THREADS;
  const int first_of = c.sh_tok[2 * MK_MAX_TOKENS + lane];
  barrier_wait(c);
  const E *w = (const E *)st.conv_w;
  for (int i = mx_spread(c); i < M * (per + hper); i += c.G) {
    if (i >= M * per) {
      const int k = i - M * per, t = k / hper, h = (k - t * hper) * MK_THREADS + threadIdx.x;
      if (h >= H) continue;
      const float z = fx_ldc((const E *)st.in + (size_t)t * st.ld_in + st.cols[1] + h) + st.step_bias[h];
      const float dt = z > 20.f ? z : log1pf(expf(z));
      float *o = (float *)st.out2 + (size_t)t * st.ld_out2 + h;
      stc_f32(o, dt);
      stc_f32(o + st.cols[2], exp2f(st.a_tab[h] * dt));
      continue;
    }
    const int t = i / per, q = (i - t * per) * MK_THREADS + threadIdx.x;
    const int t0 = __builtin_amdgcn_readfirstlane(c.sh_tok[2 * MK_MAX_TOKENS + t]), p0 = __builtin_amdgcn_readfirstlane(c.sh_tok[t0]), lead = t - t0;
    const int cnt = __popcll(__ballot(lane < M && first_of == t0));  // the request's tokens
    if (q >= n4 || (lead > 0 && lead < taps - 1)) continue;
    E *ring = (E *)st.tail + (size_t)__builtin_amdgcn_readfirstlane(c.state_ids[__builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + t])]) * taps * n + 4 * q;
    const E *x = (const E *)st.in + st.cols[0] + 4 * q;
    f32x4 bias = {0.f, 0.f, 0.f, 0.f};
    if (st.in_bias) bias = *(const f32x4 *)(st.in_bias + 4 * q);
    auto put = [&](int u, f32x4 acc) {
      if (st.flags & MK_F_SILU) {
#pragma unroll
        for (int e = 0; e < 4; e++) acc[e] = hy_silu(E(), acc[e]);
      }
      fx_stc_quad((E *)st.out + (size_t)u * st.ld_out + 4 * q, acc);
    };
    if (lead == 0 && taps <= 4) {  // few taps: everything is requested at once
      const int lo = max(t0, t0 + cnt - (taps - 1));
      f32x4 v[6], g[4], last[3];  // v[r]: input at position p0 - 3 + r
#pragma unroll
      for (int r = 0; r < 6; r++) {
        const bool old = r < 3 && 3 - r < taps && p0 - 3 + r >= 0;
        v[r] = fx_ldc_quad(old ? ring + (size_t)((p0 - 3 + r) % taps) * n : x + (size_t)(t0 + min(max(r - 3, 0), cnt - 1)) * st.ld_in);
      }
#pragma unroll
      for (int b = 0; b < 4; b++) g[b] = fx_ld_quad(w + (size_t)(taps - 1 - min(b, taps - 1)) * n + 4 * q);
#pragma unroll
      for (int r = 0; r < 3; r++) last[r] = fx_ldc_quad(x + (size_t)min(lo + r, t0 + cnt - 1) * st.ld_in);
#pragma unroll
      for (int u = 0; u < 3; u++) {
        if (u >= min(cnt, max(taps - 1, 1))) break;
        f32x4 acc = bias;
#pragma unroll
        for (int b = 0; b < 4; b++)
#pragma unroll
          for (int e = 0; e < 4; e++) acc[e] = b < taps && b <= p0 + u ? fmaf(v[3 + u - b][e], g[b][e], acc[e]) : acc[e];
        if (st.flags & MK_F_IDENTITY) acc += v[3 + u];
        put(t0 + u, acc);
      }
#pragma unroll
      for (int r = 0; r < 3; r++)
        if (lo + r < t0 + cnt && r < taps - 1) fx_stc_quad(ring + (size_t)((p0 + lo + r - t0) % taps) * n, last[r]);
      continue;
    }
    const int t1 = lead == 0 ? t0 + min(cnt, max(taps - 1, 1)) : t + 1;  // tokens [t, t1)
    for (int u = t; u < t1; u++) {
      const int pos = p0 + u - t0;
      f32x4 acc = bias;
      for (int b0 = 0; b0 < taps; b0 += 4) {  // b: positions back
        f32x4 v[4], g[4];
#pragma unroll
        for (int y = 0; y < 4; y++) {
          const int b = min(b0 + y, taps - 1);
          v[y] = fx_ldc_quad(b > u - t0 ? ring + (size_t)(max(pos - b, 0) % taps) * n : x + (size_t)(u - b) * st.ld_in);
          g[y] = fx_ld_quad(w + (size_t)(taps - 1 - b) * n + 4 * q);
        }
#pragma unroll
        for (int y = 0; y < 4; y++) {
          const bool on = b0 + y < taps && b0 + y <= pos;
#pragma unroll
          for (int e = 0; e < 4; e++) acc[e] = on ? fmaf(v[y][e], g[y][e], acc[e]) : acc[e];
          if (b0 + y == 0 && (st.flags & MK_F_IDENTITY)) acc += v[y];
        }
      }
      put(u, acc);
    }
    if (lead == 0) {  // the request's last inputs (the ring's rows have been read)
      for (int u = max(t0, t0 + cnt - (taps - 1)); u < t0 + cnt; u++) fx_stc_quad(ring + (size_t)((p0 + u - t0) % taps) * n, fx_ldc_quad(x + (size_t)u * st.ld_in));
    }
  }
  c.wrote_through = true;
}

// ----------------------------------------------------------------------------- recurrence per head
// A state is [head][value][states rounded up to 4], fp32.  L = 4, 8 or 16 lanes hold the states of one value, Q quads each (lane j of
// them states 4 (i L + j) .. + 3, i < Q), so the sum over states stays among L neighbours; a lane works on CH values at a time.  A unit is
// a request's head and 256 CH / L of its values; step, decay, B and C of a token are the same for all of it.
// in: projection rows (z from column cols[3] on), q_ws: convolved rows (x from cols[0], B from cols[1], C from cols[2] on; a group's
// B and C take the padded number of states), in2: steps and, from column cols[4] on, decays, out: 32-bit rows.
struct DuUnit {
  int h, v0, t0, n, p0;
  float *state;
};
template <int CH>
__device__ __forceinline__ DuUnit du_unit(CStage &st, const Ctx &c, const MkRuntime &rt, const MxDeltaUnits &us, int u, int lg2) {
  const int GW = 64 >> lg2, CW = MK_WAVES * GW * CH, V = st.v_dim, H = st.num_q_heads, Np = (st.states + 3) / 4 * 4, nblk = (V + CW - 1) / CW;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), uh = u / nblk, ri = uh / H;
  DuUnit a;
  a.h = uh - ri * H;
  a.v0 = (u - uh * nblk) * CW + wave * GW * CH + (lane >> lg2);
  a.t0 = (int)__ffsll(__ballot(us.first && us.rank_of == ri)) - 1;
  a.n = wave_bcast(us.my_n, a.t0);
  a.p0 = __builtin_amdgcn_readfirstlane(c.sh_tok[a.t0]);
  a.state = (float *)st.k_cache + ((size_t)__builtin_amdgcn_readfirstlane(rt.state_ids[__builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + a.t0])]) * H + a.h) * V * Np;
  return a;
}
// Where a lane's quads of states lie; values behind the last and quads behind the last repeat one (computed, not stored).
template <int Q>
struct DuLanes {
  int at[Q], GW, V, Np;
  bool on[Q];
  __device__ __forceinline__ DuLanes(CStage &st, int lg2) {
    const int L = 1 << lg2, j = threadIdx.x & (L - 1);
    GW = 64 >> lg2;
    V = st.v_dim;
    Np = (st.states + 3) / 4 * 4;
#pragma unroll
    for (int i = 0; i < Q; i++) {
      on[i] = 4 * (i * L + j) < Np;
      at[i] = min(4 * (i * L + j), Np - 4);
    }
  }
  __device__ __forceinline__ int value(const DuUnit &a, int h) const { return min(a.v0 + h * GW, V - 1); }
  __device__ __forceinline__ bool real(const DuUnit &a, int h) const { return a.v0 + h * GW < V; }
  template <int CH>
  __device__ __forceinline__ void load(const DuUnit &a, f32x4 (&S)[CH][Q]) const {
#pragma unroll
    for (int h = 0; h < CH; h++)
#pragma unroll
      for (int i = 0; i < Q; i++) S[h][i] = __builtin_nontemporal_load((const f32x4 *)(a.state + (size_t)value(a, h) * Np + at[i]));
  }
  template <int CH>
  __device__ __forceinline__ void clear(const DuUnit &a, f32x4 (&S)[CH][Q]) const {
#pragma unroll
    for (int h = 0; h < CH; h++)
#pragma unroll
      for (int i = 0; i < Q; i++)
        if (!on[i] || a.p0 == 0) S[h][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }
  // written through, 16 bytes a store, by an instruction whose completion the compiler counts (it cannot for inline assembly, and a
  // wait for a later load would then wait for the stores too)
  template <int CH>
  __device__ __forceinline__ void store(const DuUnit &a, const f32x4 (&S)[CH][Q]) const {
    const __amdgpu_buffer_rsrc_t rs = __builtin_amdgcn_make_buffer_rsrc(a.state, 0, V * Np * 4, 0x00027000);
#pragma unroll
    for (int h = 0; h < CH; h++)
#pragma unroll
      for (int i = 0; i < Q; i++)
        if (on[i] && real(a, h)) __builtin_amdgcn_raw_buffer_store_b128(__builtin_bit_cast(u32x4, S[h][i]), rs, (value(a, h) * Np + at[i]) * 4, 0, 16);
  }
};
// one token: S <- da S + (dt x) B, returns S C
template <int Q>
__device__ __forceinline__ float du_step(f32x4 (&S)[Q], const f32x4 (&B)[Q], const f32x4 (&C)[Q], float dx, float da, int L) {
  f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < Q; i++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      S[i][e] = fmaf(da, S[i][e], dx * B[i][e]);
      s[e] = fmaf(S[i][e], C[i][e], s[e]);
    }
  return hy_lanes_sum((s[0] + s[1]) + (s[2] + s[3]), L);
}
// every request brings one token: the states of the next DEP units are in flight while one is computed
template <typename E, int Q, int CH, int DEP>
__device__ __forceinline__ void stage_du_scan_single(CStage &st, Ctx &c, const MkRuntime &rt, int M, int lg2) {
  static_assert(DEP == 1 || DEP == 2, "");
  static_assert(CH <= 4, "a lane finishes one output, four lanes or more share a value");
  const int L = 1 << lg2, j = threadIdx.x & (L - 1), CW = MK_WAVES * (64 >> lg2) * CH;
  const int V = st.v_dim, H = st.num_q_heads, per_group = H / st.groups, nblk = (V + CW - 1) / CW;
  const DuLanes<Q> ln(st, lg2);
  const MxDeltaUnits us = mx_delta_units(c, M);
  const int n_units = us.nreq * H * nblk;
  struct Rows {
    f32x4 B[Q], C[Q];
    float dt, da, x[CH], z;
  };
  auto load_rows = [&](const DuUnit &a, Rows &r) {
    const E *row = (const E *)st.q_ws + (size_t)a.t0 * st.ld_qws;
    const float *steps = (const float *)st.in2 + (size_t)a.t0 * st.ld_in2;
    const int g = a.h / per_group * ln.Np;
#pragma unroll
    for (int i = 0; i < Q; i++) {
      r.B[i] = fx_ldc_quad(row + st.cols[1] + g + ln.at[i]);
      r.C[i] = fx_ldc_quad(row + st.cols[2] + g + ln.at[i]);
    }
    r.dt = ldc_f32(steps + a.h);
    r.da = ldc_f32(steps + st.cols[4] + a.h);
#pragma unroll
    for (int h = 0; h < CH; h++) r.x[h] = fx_ldc(row + st.cols[0] + a.h * V + ln.value(a, h));
    r.z = fx_ldc((const E *)st.in + (size_t)a.t0 * st.ld_in + st.cols[3] + a.h * V + ln.value(a, min(j, CH - 1)));
  };
  const int u0 = mx_spread(c);
  const bool have = u0 < n_units, early = have && threadIdx.x >= 64;
  auto unit = [&](int u) { return du_unit<CH>(st, c, rt, us, min(u, n_units - 1 - (n_units - 1 - u0) % c.G), lg2); };  // (behind the last: the last again)
  // A ring of DEP + 1 units, unrolled so that registers which still wait for their loads are never copied.
  f32x4 S[DEP + 1][CH][Q];
  Rows r[DEP + 1];
  DuUnit a[DEP + 1];
  if (have) {
#pragma unroll
    for (int d = 0; d <= DEP; d++) a[d] = unit(u0 + d * c.G);
  }
  // earlier iterations wrote the states: the first ones are requested before the barrier is awaited
  if (early) {
#pragma unroll
    for (int d = 0; d < DEP; d++) ln.template load<CH>(a[d], S[d]);
  }
  barrier_wait(c);
  c.wrote_through = true;
  if (!have) return;
#pragma unroll
  for (int d = 0; d < DEP; d++) {
    if (!early) ln.template load<CH>(a[d], S[d]);
    load_rows(a[d], r[d]);
  }
  auto step = [&](int u, auto slot) {
    constexpr int I = decltype(slot)::value, F = (I + DEP) % (DEP + 1);
    a[F] = unit(u + DEP * c.G);
    load_rows(a[F], r[F]);
    ln.template load<CH>(a[F], S[F]);
    const float D = st.d_tab[a[I].h];
    ln.template clear<CH>(a[I], S[I]);
#pragma unroll
    for (int i = 0; i < Q; i++)
      if (!ln.on[i]) r[I].B[i] = r[I].C[i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    float y = 0.f;
#pragma unroll
    for (int h = 0; h < CH; h++) {
      const float s = du_step<Q>(S[I][h], r[I].B, r[I].C, r[I].dt * r[I].x[h], r[I].da, L) + D * r[I].x[h];
      y = j == h ? s : y;
    }
    if (j < CH && ln.real(a[I], j)) stc_f32((float *)st.out + (size_t)a[I].t0 * st.ld_out + a[I].h * V + ln.value(a[I], j), y * hy_silu(E(), r[I].z));
    ln.template store<CH>(a[I], S[I]);
  };
  for (int u = u0;;) {
    step(u, std::integral_constant<int, 0>{});
    if ((u += c.G) >= n_units) break;
    step(u, std::integral_constant<int, 1>{});
    if ((u += c.G) >= n_units) break;
    if constexpr (DEP == 2) {
      step(u, std::integral_constant<int, 2>{});
      if ((u += c.G) >= n_units) break;
    }
  }
}
// some request brings several tokens: the rows of a unit's portion are put in LDS at once (32-bit), then every group of lanes walks them
template <typename E, int Q, int CH>
__device__ __forceinline__ void stage_du_scan_portions(CStage &st, Ctx &c, const MkRuntime &rt, int M, int lg2, char *smem) {
  const int L = 1 << lg2, GW = 64 >> lg2, CW = MK_WAVES * GW * CH, tid = threadIdx.x, lane = tid & 63, j = lane & (L - 1), wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int V = st.v_dim, H = st.num_q_heads, per_group = H / st.groups, nblk = (V + CW - 1) / CW;
  const DuLanes<Q> ln(st, lg2);
  const int Np = 4 * L * Q, n4 = Np / 4, real4 = ln.Np / 4;  // (rows in LDS are padded with zeros to what the lanes read)
  const MxDeltaUnits us = mx_delta_units(c, M);
  const int n_units = us.nreq * H * nblk;
  float *Bs = (float *)smem, *Cs = Bs + MK_MAX_TOKENS * Np, *ds = Cs + MK_MAX_TOKENS * Np, *Xs = ds + 2 * MK_MAX_TOKENS;  // [token][states] x 2, steps, decays, [token][CW]
  const int u0 = mx_spread(c);
  f32x4 S[CH][Q];
  DuUnit a{};
  const bool early = u0 < n_units && wave != 0;
  if (u0 < n_units) a = du_unit<CH>(st, c, rt, us, u0, lg2);
  if (early) ln.template load<CH>(a, S);
  barrier_wait(c);
  for (int u = u0; u < n_units; u += c.G) {
    if (u != u0) a = du_unit<CH>(st, c, rt, us, u, lg2);
    if (!(u == u0 && early)) ln.template load<CH>(a, S);
    const int vb = (u % nblk) * CW, g = a.h / per_group * ln.Np, nx = min(CW, V - vb);
    const E *rows = (const E *)st.q_ws + (size_t)a.t0 * st.ld_qws;
    __syncthreads();  // LDS reuse
    for (int i0 = tid; i0 < a.n * 2 * n4; i0 += 8 * MK_THREADS) {
      f32x4 v[8];
#pragma unroll
      for (int y = 0; y < 8; y++) {
        const int i = min(i0 + y * MK_THREADS, a.n * 2 * n4 - 1), t = i / (2 * n4), k = i - t * 2 * n4;
        const int q = k < n4 ? k : k - n4;
        v[y] = fx_ldc_quad(rows + (size_t)t * st.ld_qws + g + st.cols[k < n4 ? 1 : 2] + 4 * min(q, real4 - 1));
        if (q >= real4) v[y] = (f32x4){0.f, 0.f, 0.f, 0.f};
      }
#pragma unroll
      for (int y = 0; y < 8; y++) {
        const int i = i0 + y * MK_THREADS, t = i / (2 * n4), k = i - t * 2 * n4;
        if (i < a.n * 2 * n4) *(f32x4 *)((k < n4 ? Bs + t * Np + 4 * k : Cs + t * Np + 4 * (k - n4))) = v[y];
      }
    }
    for (int i0 = tid; i0 < a.n * CW; i0 += 8 * MK_THREADS) {
      float v[8];
#pragma unroll
      for (int y = 0; y < 8; y++) {
        const int i = min(i0 + y * MK_THREADS, a.n * CW - 1), t = i / CW, k = i - t * CW;
        v[y] = fx_ldc(rows + (size_t)t * st.ld_qws + st.cols[0] + a.h * V + vb + min(k, nx - 1));
      }
#pragma unroll
      for (int y = 0; y < 8; y++)
        if (i0 + y * MK_THREADS < a.n * CW) Xs[i0 + y * MK_THREADS] = v[y];
    }
    if (tid < 2 * a.n) {
      const int t = tid >> 1;
      ds[tid] = ldc_f32((const float *)st.in2 + (size_t)(a.t0 + t) * st.ld_in2 + (tid & 1 ? st.cols[4] : 0) + a.h);
    }
    const float D = st.d_tab[a.h];
    ln.template clear<CH>(a, S);
    __syncthreads();
    struct Vec {
      f32x4 B[Q], C[Q];
      float dt, da, x[CH];
    };
    const int xv = wave * GW * CH + (lane >> lg2);
    auto load_vec = [&](int t, Vec &r) {
#pragma unroll
      for (int i = 0; i < Q; i++) {
        r.B[i] = *(const f32x4 *)(Bs + t * Np + 4 * (i * L + j));
        r.C[i] = *(const f32x4 *)(Cs + t * Np + 4 * (i * L + j));
      }
      r.dt = ds[2 * t];
      r.da = ds[2 * t + 1];
#pragma unroll
      for (int h = 0; h < CH; h++) r.x[h] = Xs[t * CW + xv + h * GW];
    };
    auto step = [&](int t, Vec &r, Vec &next) {  // (the next token's values are fetched meanwhile)
      load_vec(min(t + 1, a.n - 1), next);
#pragma unroll
      for (int h = 0; h < CH; h++) {
        const float s = du_step<Q>(S[h], r.B, r.C, r.dt * r.x[h], r.da, L) + D * r.x[h];
        if (j == h) Xs[t * CW + xv + h * GW] = s;  // (the value's input has been read by all of its lanes)
      }
    };
    Vec r0, r1;
    load_vec(0, r0);
    for (int t = 0;;) {
      step(t, r0, r1);
      if (++t >= a.n) break;
      step(t, r1, r0);
      if (++t >= a.n) break;
    }
    ln.template store<CH>(a, S);
    __syncthreads();
    for (int i0 = tid; i0 < a.n * CW; i0 += 8 * MK_THREADS) {
      float z[8];
#pragma unroll
      for (int y = 0; y < 8; y++) {
        const int i = min(i0 + y * MK_THREADS, a.n * CW - 1), t = i / CW, k = i - t * CW;
        z[y] = fx_ldc((const E *)st.in + (size_t)(a.t0 + t) * st.ld_in + st.cols[3] + a.h * V + vb + min(k, nx - 1));
      }
#pragma unroll
      for (int y = 0; y < 8; y++) {
        const int i = i0 + y * MK_THREADS, t = i / CW, k = i - t * CW;
        if (i < a.n * CW && k < nx) stc_f32((float *)st.out + (size_t)(a.t0 + t) * st.ld_out + a.h * V + vb + k, Xs[i] * hy_silu(E(), z[y]));
      }
    }
  }
  c.wrote_through = true;
}
template <typename E, int Q>
__device__ __forceinline__ void stage_du_scan_q(CStage &st, Ctx &c, const MkRuntime &rt, int M, bool single, int lg2, char *smem) {
  const long long values = (long long)st.num_q_heads * st.v_dim;
  if (single) {
    if (((M * values) << lg2) >= 4ll * c.G * MK_THREADS) stage_du_scan_single<E, Q, 4, Q == 4 ? 1 : 2>(st, c, rt, M, lg2);
    else stage_du_scan_single<E, Q, 1, 1>(st, c, rt, M, lg2);
  } else if (((mx_delta_units(c, M).nreq * values) << lg2) > (long long)c.G * MK_THREADS) {
    stage_du_scan_portions<E, Q, 2>(st, c, rt, M, lg2, smem);
  } else {
    stage_du_scan_portions<E, Q, 1>(st, c, rt, M, lg2, smem);
  }
}
template <typename E>
__device__ __forceinline__ void stage_du_scan(CStage &st, Ctx &c, const MkRuntime &rt, int M, bool single, char *smem) {
  static_assert((2 * MK_MAX_TOKENS * MK_HY_MAX_STATES + 2 * MK_MAX_TOKENS + MK_MAX_TOKENS * 2 * MK_WAVES * 4) * 4 <= MK_LDS_BYTES, "rows of a portion fit in LDS");
  const int lg2 = st.states <= 16 ? 2 : st.states <= 32 ? 3 : 4;
  if (st.states <= 64) stage_du_scan_q<E, 1>(st, c, rt, M, single, lg2, smem);
  else if (st.states <= 128) stage_du_scan_q<E, 2>(st, c, rt, M, single, lg2, smem);
  else stage_du_scan_q<E, 4>(st, c, rt, M, single, lg2, smem);
}
