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
  const int n = st.n, n4 = n / 4, taps = st.taps, per = (n4 + MK_THREADS - 1) / MK_THREADS;
  const int H = st.step_bias ? st.num_q_heads : 0, hper = (H + MK_THREADS - 1) / MK_THREADS;
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
    if (q >= n4 || (lead > 0 && lead < taps - 1)) continue;
    int t1 = t + 1;  // tokens [t, t1)
    if (lead == 0) {
      while (t1 < M && t1 - t0 < taps - 1 && __builtin_amdgcn_readfirstlane(c.sh_tok[2 * MK_MAX_TOKENS + t1]) == t0) t1++;
    }
    E *ring = (E *)st.tail + (size_t)__builtin_amdgcn_readfirstlane(c.state_ids[__builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + t])]) * taps * n + 4 * q;
    const E *x = (const E *)st.in + st.cols[0] + 4 * q;
    f32x4 bias = {0.f, 0.f, 0.f, 0.f};
    if (st.in_bias) bias = *(const f32x4 *)(st.in_bias + 4 * q);
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
      if (st.flags & MK_F_SILU) {
#pragma unroll
        for (int e = 0; e < 4; e++) acc[e] = hy_silu(E(), acc[e]);
      }
      fx_stc_quad((E *)st.out + (size_t)u * st.ld_out + 4 * q, acc);
    }
    if (lead == 0) {  // the request's last inputs (the ring's rows have been read)
      int end = t1;
      while (end < M && __builtin_amdgcn_readfirstlane(c.sh_tok[2 * MK_MAX_TOKENS + end]) == t0) end++;
      for (int u = max(t0, end - (taps - 1)); u < end; u++) fx_stc_quad(ring + (size_t)((p0 + u - t0) % taps) * n, fx_ldc_quad(x + (size_t)u * st.ld_in));
    }
  }
  c.wrote_through = true;
}

// ----------------------------------------------------------------------------- recurrence per head
// A state is [head][value][states rounded up to 4], fp32.  L = 4, 8 or 16 lanes hold the states of one value, Q quads each (lane j of
// them states 4 (i L + j) .. + 3, i < Q), so the sum over states stays among L neighbours; a lane works on CH values at a time.  A unit is
// a request's head and 256 CH / L of its values; step, decay, B and C of a token are the same for all of it.  It walks the request's tokens, TB at a
// time, the next TB (or the next unit with its state) in flight meanwhile; a lane finishes (gate, store) one output.
// in: projection rows (z from column cols[3] on), q_ws: convolved rows (x from cols[0], B from cols[1], C from cols[2] on; a group's
// B and C take the padded number of states), in2: steps and, from column cols[4] on, decays, out: 32-bit rows.
template <typename E, int Q, int TB, int CH>
__device__ __forceinline__ void stage_du_scan_t(CStage &st, Ctx &c, const MkRuntime &rt, int M, int lg2) {
  static_assert(TB * CH <= 4, "a lane finishes one output, four lanes or more share a value");
  const int L = 1 << lg2, GW = 64 >> lg2, CW = MK_WAVES * GW * CH;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), j = lane & (L - 1);
  const int V = st.v_dim, H = st.num_q_heads, per_group = H / st.groups, Np = (st.states + 3) / 4 * 4, nblk = (V + CW - 1) / CW;
  const MxDeltaUnits us = mx_delta_units(c, M);
  const int n_units = us.nreq * H * nblk;
  const E *in = (const E *)st.in, *xc = (const E *)st.q_ws;
  const float *steps = (const float *)st.in2;
  struct Unit {
    int h, v0, t0, n, p0;
    float *state;
  };
  auto unit = [&](int u) {
    Unit a;
    const int uh = u / nblk, ri = uh / H;
    a.h = uh - ri * H;
    a.v0 = (u - uh * nblk) * CW + wave * GW * CH + (lane >> lg2);
    a.t0 = (int)__ffsll(__ballot(us.first && us.rank_of == ri)) - 1;
    a.n = wave_bcast(us.my_n, a.t0);
    a.p0 = __builtin_amdgcn_readfirstlane(c.sh_tok[a.t0]);
    a.state = (float *)st.k_cache + ((size_t)__builtin_amdgcn_readfirstlane(rt.state_ids[__builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + a.t0])]) * H + a.h) * V * Np;
    return a;
  };
  auto value = [&](const Unit &a, int h) { return min(a.v0 + h * GW, V - 1); };  // (behind the last: computed, not stored)
  auto real = [&](const Unit &a, int h) { return a.v0 + h * GW < V; };
  int at[Q];
  bool on[Q];
#pragma unroll
  for (int i = 0; i < Q; i++) {
    on[i] = 4 * (i * L + j) < Np;
    at[i] = min(4 * (i * L + j), Np - 4);
  }
  auto load_state = [&](const Unit &a, f32x4 (&S)[CH][Q]) {
#pragma unroll
    for (int h = 0; h < CH; h++)
#pragma unroll
      for (int i = 0; i < Q; i++) S[h][i] = __builtin_nontemporal_load((const f32x4 *)(a.state + (size_t)value(a, h) * Np + at[i]));
  };
  struct Rows {
    f32x4 B[TB][Q], C[TB][Q];
    float dt[TB], da[TB], x[TB][CH], z;
  };
  auto load_rows = [&](const Unit &a, int tb, Rows &r) {
    const int g = a.h / per_group;
#pragma unroll
    for (int t = 0; t < TB; t++) {
      const size_t tok = a.t0 + min(tb + t, a.n - 1);
      const E *row = xc + tok * st.ld_qws;
#pragma unroll
      for (int i = 0; i < Q; i++) {
        r.B[t][i] = fx_ldc_quad(row + st.cols[1] + g * Np + at[i]);
        r.C[t][i] = fx_ldc_quad(row + st.cols[2] + g * Np + at[i]);
      }
      r.dt[t] = ldc_f32(steps + tok * st.ld_in2 + a.h);
      r.da[t] = ldc_f32(steps + tok * st.ld_in2 + st.cols[4] + a.h);
#pragma unroll
      for (int h = 0; h < CH; h++) r.x[t][h] = fx_ldc(row + st.cols[0] + a.h * V + value(a, h));
    }
    const int e = min(j, TB * CH - 1);
    r.z = fx_ldc(in + (size_t)(a.t0 + min(tb + e / CH, a.n - 1)) * st.ld_in + st.cols[3] + a.h * V + value(a, e % CH));
  };
  const int u0 = mx_spread(c);
  f32x4 S[CH][Q];
  Unit a{};
  // earlier iterations wrote the state: the first unit's is requested before the barrier is awaited
  const bool early = u0 < n_units && wave != 0;
  if (u0 < n_units) a = unit(u0);
  if (early) load_state(a, S);
  barrier_wait(c);
  if (u0 < n_units && !early) load_state(a, S);
  Rows r;
  if (u0 < n_units) load_rows(a, 0, r);
  for (int u = u0; u < n_units; u += c.G) {
    const Unit nx = u + c.G < n_units ? unit(u + c.G) : a;
    f32x4 Sn[CH][Q];
    load_state(nx, Sn);
    const float D = st.d_tab[a.h];
#pragma unroll
    for (int h = 0; h < CH; h++)
#pragma unroll
      for (int i = 0; i < Q; i++)
        if (!on[i] || a.p0 == 0) S[h][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int tb = 0; tb < a.n; tb += TB) {
      Rows rn;
      const bool more = tb + TB < a.n;
      load_rows(more ? a : nx, more ? tb + TB : 0, rn);
      float y = 0.f;
#pragma unroll
      for (int t = 0; t < TB; t++) {
        if (TB > 1 && tb + t >= a.n) break;
#pragma unroll
        for (int h = 0; h < CH; h++) {
          const float dx = r.dt[t] * r.x[t][h];
          float s = 0.f;
#pragma unroll
          for (int i = 0; i < Q; i++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
              S[h][i][e] = fmaf(r.da[t], S[h][i][e], on[i] ? dx * r.B[t][i][e] : 0.f);
              s = fmaf(S[h][i][e], on[i] ? r.C[t][i][e] : 0.f, s);
            }
          s = hy_lanes_sum(s, L) + D * r.x[t][h];
          y = j == t * CH + h ? s : y;
        }
      }
      const int t = j / CH, h = j % CH;
      if (j < TB * CH && tb + t < a.n && real(a, h)) stc_f32((float *)st.out + (size_t)(a.t0 + tb + t) * st.ld_out + a.h * V + value(a, h), y * hy_silu(E(), r.z));
      r = rn;
    }
#pragma unroll
    for (int h = 0; h < CH; h++) {
      if (!real(a, h)) continue;
#pragma unroll
      for (int i = 0; i < Q; i++)
        if (on[i]) mx_stc_quad(a.state + (size_t)value(a, h) * Np + at[i], S[h][i]);
    }
    a = nx;
#pragma unroll
    for (int h = 0; h < CH; h++)
#pragma unroll
      for (int i = 0; i < Q; i++) S[h][i] = Sn[h][i];
  }
  c.wrote_through = true;
}
template <typename E, int Q>
__device__ __forceinline__ void stage_du_scan_q(CStage &st, Ctx &c, const MkRuntime &rt, int M, bool single, int lg2) {
  if (!single) stage_du_scan_t<E, Q, 4, 1>(st, c, rt, M, lg2);
  else if ((((long long)M * st.num_q_heads * st.v_dim) << lg2) >= 2ll * c.G * MK_THREADS) stage_du_scan_t<E, Q, 1, 4>(st, c, rt, M, lg2);
  else stage_du_scan_t<E, Q, 1, 1>(st, c, rt, M, lg2);
}
template <typename E>
__device__ __forceinline__ void stage_du_scan(CStage &st, Ctx &c, const MkRuntime &rt, int M, bool single) {
  const int lg2 = st.states <= 16 ? 2 : st.states <= 32 ? 3 : 4;
  if (st.states <= 64) stage_du_scan_q<E, 1>(st, c, rt, M, single, lg2);
  else if (st.states <= 128) stage_du_scan_q<E, 2>(st, c, rt, M, single, lg2);
  else stage_du_scan_q<E, 4>(st, c, rt, M, single, lg2);
}
