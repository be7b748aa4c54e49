// Selective scan and expert feed-forwards (part of the persistent kernel, included by mk_kernel.hip behind mk_flex.hip and
// mk_mix.hip, whose conventions it keeps: sizes and constants are descriptor fields, E is the type of activations and weights,
// everything named in 32 bits is 32-bit in both builds).
//   * stage_hy_conv     causal convolution per channel and silu, the inputs before the portion come from the request's slot;
//   * stage_hy_scan     S' = exp(dt A) S + dt x B, y = (S' C + D x) silu(z), state and convolution tail per request;
//   * stage_hy_route    softmax over experts, the largest few, their shares;
//   * stage_hy_experts  gated or plain linears of the chosen experts over their tokens, and of a shared expert over all tokens.
// (The step sizes dt and the router logits are forms of stage_mx_head_linear, the weighted sum over a token's experts is part of
// the norm behind it.)

__device__ __forceinline__ float hy_silu(uint16_t, float z) { return z * mx_sigmoid((uint16_t)0, z); }
__device__ __forceinline__ float hy_silu(float, float z) { return z / (1.f + expf(-z)); }

// ----------------------------------------------------------------------------- convolution
// out[t, c] = silu(b[c] + sum_j w[j][c] x[t - (taps - 1) + j, c]); st.n channels (a multiple of 4), x = in[t, cols[0] + c], w fp32
// [taps][n].  Tail of a slot: [taps - 1][n], row r the input at position p0 - (taps - 1) + r; positions before the first count as
// zero whatever the slot holds.  The scan stage writes the new tail, so that every token of a portion is independent here.
template <typename E>
__device__ __forceinline__ void stage_hy_conv(CStage &st, Ctx &c, const MkRuntime &rt, int M) {
  barrier_wait(c);
  const int n = st.n, n4 = n / 4, taps = st.taps, per = (n4 + MK_THREADS - 1) / MK_THREADS;
  const float *w = (const float *)st.norm_w;
  for (int i = mx_spread(c); i < M * per; i += c.G) {
    const int t = i / per, q = (i - t * per) * MK_THREADS + threadIdx.x;
    if (q >= n4) continue;
    const int t0 = __builtin_amdgcn_readfirstlane(c.sh_tok[2 * MK_MAX_TOKENS + t]), pos = __builtin_amdgcn_readfirstlane(c.sh_tok[t]);
    const int slot = __builtin_amdgcn_readfirstlane(rt.state_ids[__builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + t])]);
    const E *x = (const E *)st.in + st.cols[0] + 4 * q, *tail = (const E *)st.tail + (size_t)slot * (taps - 1) * n + 4 * q;
    f32x4 acc = *(const f32x4 *)(st.in_bias + 4 * q);
    for (int j0 = 0; j0 < taps; j0 += 4) {
      f32x4 v[4], g[4];
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const int tap = min(j0 + j, taps - 1), back = taps - 1 - tap, k = back - (t - t0);  // k > 0: k positions before the portion
        const E *src = k > 0 ? tail + (size_t)(taps - 1 - k) * n : x + (size_t)(t - back) * st.ld_in;
        v[j] = fx_ldc_quad(src);
        g[j] = *(const f32x4 *)(w + (size_t)tap * n + 4 * q);
      }
#pragma unroll
      for (int j = 0; j < 4; j++) {
        const bool on = j0 + j < taps && taps - 1 - (j0 + j) <= pos;
#pragma unroll
        for (int e = 0; e < 4; e++) acc[e] = on ? fmaf(v[j][e], g[j][e], acc[e]) : acc[e];
      }
    }
#pragma unroll
    for (int e = 0; e < 4; e++) acc[e] = hy_silu(E(), acc[e]);
    fx_stc_quad((E *)st.out + (size_t)t * st.ld_out + 4 * q, acc);
  }
  c.wrote_through = true;
}

// ----------------------------------------------------------------------------- selective scan
// L = 4, 8 or 16 lanes hold the states of a channel, Q quads each: lane j of them states 4 (i L + j) .. + 3, i < Q, so the sum over states stays
// among L neighbours.  A lane works on CH channels at a time.  A workgroup takes 256 CH / L channels of one request and walks its
// tokens, TB at a time; the rows of the next TB (or of the next unit, with its state) are in flight meanwhile.  A lane finishes (gate,
// store) every L-th output.  State: fp32 [slot][channel][states rounded up to 4], zero where a request begins.  dt: fp32
// rows (in2), x: conv output rows (q_ws), B and C: columns cols[1], cols[2] of in3, z: column cols[3] of in.
__device__ __forceinline__ float hy_lanes_sum(float v, int L) {
  v += dpp_f32<0xB1>(v);  // quad_perm [1,0,3,2]
  v += dpp_f32<0x4E>(v);  // quad_perm [2,3,0,1]
  v += L >= 8 ? dpp_f32<0x141>(v) : 0.f;   // row_half_mirror
  v += L >= 16 ? dpp_f32<0x140>(v) : 0.f;  // row_mirror
  return v;
}
template <typename E, int Q, int TB, int CH>
__device__ __forceinline__ void stage_hy_scan_t(CStage &st, Ctx &c, const MkRuntime &rt, int M, int lg2) {
  constexpr int KK = (TB * CH + 3) / 4;  // (outputs a lane finishes, with the fewest lanes per channel)
  const int L = 1 << lg2, GW = 64 >> lg2, CW = MK_WAVES * GW * CH;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), j = lane & (L - 1);
  const int n = st.n, Np = (st.states + 3) / 4 * 4, nblk = (n + CW - 1) / CW;
  const MxDeltaUnits us = mx_delta_units(c, M);
  const int n_units = us.nreq * nblk;
  const E *in = (const E *)st.in, *xc = (const E *)st.q_ws, *bc = (const E *)st.in3;
  const float *dtr = (const float *)st.in2;
  struct Unit {
    int ch0, t0, n, p0, slot;
  };
  auto unit = [&](int u) {
    Unit a;
    const int ri = u / nblk;
    a.ch0 = (u - ri * nblk) * CW + wave * GW * CH + (lane >> lg2);
    a.t0 = (int)__ffsll(__ballot(us.first && us.rank_of == ri)) - 1;
    a.n = wave_bcast(us.my_n, a.t0);
    a.p0 = __builtin_amdgcn_readfirstlane(c.sh_tok[a.t0]);
    a.slot = __builtin_amdgcn_readfirstlane(rt.state_ids[__builtin_amdgcn_readfirstlane(c.sh_tok[MK_MAX_TOKENS + a.t0])]);
    return a;
  };
  auto channel = [&](const Unit &a, int h) { return min(a.ch0 + h * GW, n - 1); };  // (behind the last: computed, not stored)
  auto real = [&](const Unit &a, int h) { return a.ch0 + h * GW < n; };
  int at[Q];
  bool on[Q];
#pragma unroll
  for (int i = 0; i < Q; i++) {
    on[i] = 4 * (i * L + j) < Np;
    at[i] = min(4 * (i * L + j), Np - 4);
  }
  auto state_of = [&](const Unit &a, int h) { return (float *)st.k_cache + ((size_t)a.slot * n + channel(a, h)) * Np; };
  auto load_state = [&](const Unit &a, f32x4 (&S)[CH][Q]) {
#pragma unroll
    for (int h = 0; h < CH; h++)
#pragma unroll
      for (int i = 0; i < Q; i++) S[h][i] = __builtin_nontemporal_load((const f32x4 *)(state_of(a, h) + at[i]));
  };
  struct Rows {
    f32x4 B[TB][Q], C[TB][Q];
    float dt[TB][CH], x[TB][CH], z[KK];
  };
  auto load_rows = [&](const Unit &a, int tb, Rows &r) {
#pragma unroll
    for (int t = 0; t < TB; t++) {
      const size_t tok = a.t0 + min(tb + t, a.n - 1);
#pragma unroll
      for (int i = 0; i < Q; i++) {
        r.B[t][i] = fx_ldc_quad(bc + tok * st.ld_in3 + st.cols[1] + at[i]);
        r.C[t][i] = fx_ldc_quad(bc + tok * st.ld_in3 + st.cols[2] + at[i]);
      }
#pragma unroll
      for (int h = 0; h < CH; h++) {
        r.dt[t][h] = ldc_f32(dtr + tok * st.ld_in2 + channel(a, h));
        r.x[t][h] = fx_ldc(xc + tok * st.ld_qws + channel(a, h));
      }
    }
#pragma unroll
    for (int k = 0; k < KK; k++)
      if (k == 0 || L == 4) r.z[k] = fx_ldc(in + (size_t)(a.t0 + min(tb + (k * L + j) / CH, a.n - 1)) * st.ld_in + st.cols[3] + channel(a, (k * L + j) % CH));
  };
  // The convolution's last inputs: the portion's, and before them what is left of the old ones.  Few taps: a lane per row, read with
  // the unit's rows and written at its end; more: in ascending order by one thread (a row is read before it is written).
  const int keep = st.taps - 1;
  auto load_tail = [&](const Unit &a, E (&v)[CH]) {
    const int i = a.n - keep + j;
#pragma unroll
    for (int h = 0; h < CH; h++) {
      const E *old = (const E *)st.tail + ((size_t)a.slot * max(keep, 1) + min(j + a.n, max(keep, 1) - 1)) * n + channel(a, h);
      v[h] = fx_round<E>(fx_ldc(i >= 0 ? in + (size_t)(a.t0 + min(i, a.n - 1)) * st.ld_in + st.cols[0] + channel(a, h) : old));
    }
  };
  f32x4 A[CH][Q];
  float D[CH];
  auto load_rates = [&](const Unit &a) {
#pragma unroll
    for (int h = 0; h < CH; h++) {
#pragma unroll
      for (int i = 0; i < Q; i++) A[h][i] = *(const f32x4 *)(st.a_tab + (size_t)channel(a, h) * Np + at[i]);
      D[h] = st.d_tab[channel(a, h)];
    }
  };
  const int u0 = mx_spread(c);
  f32x4 S[CH][Q];
  Unit a{};
  // earlier iterations wrote the state: the first unit's is requested before the barrier is awaited
  const bool early = u0 < n_units && wave != 0;
  if (u0 < n_units) a = unit(u0);
  if (early) {
    load_state(a, S);
    load_rates(a);
  }
  barrier_wait(c);
  if (u0 < n_units && !early) {
    load_state(a, S);
    load_rates(a);
  }
  Rows r;
  E tail[CH];
  if (u0 < n_units) {
    load_rows(a, 0, r);
    load_tail(a, tail);
  }
  for (int u = u0; u < n_units; u += c.G) {
    const Unit nx = u + c.G < n_units ? unit(u + c.G) : a;
    f32x4 Sn[CH][Q];
    E tail_n[CH];
    load_state(nx, Sn);
    load_tail(nx, tail_n);
#pragma unroll
    for (int h = 0; h < CH; h++)
#pragma unroll
      for (int i = 0; i < Q; i++)
        if (!on[i] || a.p0 == 0) S[h][i] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int tb = 0; tb < a.n; tb += TB) {
      Rows rn;
      const bool more = tb + TB < a.n;
      load_rows(more ? a : nx, more ? tb + TB : 0, rn);
      float y[KK];
      static_assert(TB * CH <= 8, "with more than four lanes per channel a lane finishes one output");
#pragma unroll
      for (int t = 0; t < TB; t++) {
        if (TB > 1 && tb + t >= a.n) break;
#pragma unroll
        for (int h = 0; h < CH; h++) {
          const float dx = r.dt[t][h] * r.x[t][h];
          float s = 0.f;
#pragma unroll
          for (int i = 0; i < Q; i++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
              S[h][i][e] = fmaf(fx_exp2(E(), r.dt[t][h] * A[h][i][e]), S[h][i][e], on[i] ? dx * r.B[t][i][e] : 0.f);
              s = fmaf(S[h][i][e], on[i] ? r.C[t][i][e] : 0.f, s);
            }
          s = hy_lanes_sum(s, L) + D[h] * r.x[t][h];
          const int e = t * CH + h;
          if ((e & (L - 1)) == j) {
            if (e >= 4 && L == 4) y[e / 4] = s;
            else y[0] = s;
          }
        }
      }
#pragma unroll
      for (int k = 0; k < KK; k++) {
        const int t = (k * L + j) / CH, h = (k * L + j) % CH;
        if ((k == 0 || L == 4) && t < TB && tb + t < a.n && real(a, h)) fx_stc((E *)st.out + (size_t)(a.t0 + tb + t) * st.ld_out + channel(a, h), fx_round<E>(y[k] * hy_silu(E(), r.z[k])));
      }
      r = rn;
    }
#pragma unroll
    for (int h = 0; h < CH; h++) {
      if (!real(a, h)) continue;
#pragma unroll
      for (int i = 0; i < Q; i++)
        if (on[i]) mx_stc_quad(state_of(a, h) + at[i], S[h][i]);
    }
    if (keep <= L) {
#pragma unroll
      for (int h = 0; h < CH; h++)
        if (j < keep && real(a, h)) fx_stc((E *)st.tail + ((size_t)a.slot * keep + j) * n + channel(a, h), tail[h]);
    } else if (j == 0) {
      for (int h = 0; h < CH; h++) {
        if (!real(a, h)) continue;
        E *rows = (E *)st.tail + (size_t)a.slot * keep * n + channel(a, h);
        for (int k = 0; k < keep; k++) {
          const int i = a.n - keep + k;
          fx_stc(rows + (size_t)k * n, fx_round<E>(i >= 0 ? fx_ldc(in + (size_t)(a.t0 + i) * st.ld_in + st.cols[0] + channel(a, h)) : fx_ldc(rows + (size_t)(k + a.n) * n)));
        }
      }
    }
    if (nx.ch0 != a.ch0) load_rates(nx);
    a = nx;
#pragma unroll
    for (int h = 0; h < CH; h++) {
#pragma unroll
      for (int i = 0; i < Q; i++) S[h][i] = Sn[h][i];
      tail[h] = tail_n[h];
    }
  }
  c.wrote_through = true;
}
template <typename E>
__device__ __forceinline__ void stage_hy_scan(CStage &st, Ctx &c, const MkRuntime &rt, int M, bool single) {
  const int lg2 = st.states <= 16 ? 2 : st.states <= 32 ? 3 : 4;
  // single tokens of many requests: eight channels per lane, so that a workgroup has enough in flight
  const bool many = single && (((long long)M * st.n) << lg2) >= 4ll * c.G * MK_THREADS;
  if (st.states <= 64) {
    if (many) stage_hy_scan_t<E, 1, 1, 8>(st, c, rt, M, lg2);
    else if (single) stage_hy_scan_t<E, 1, 1, 1>(st, c, rt, M, lg2);
    else stage_hy_scan_t<E, 1, 8, 1>(st, c, rt, M, lg2);
  } else {
    if (single) stage_hy_scan_t<E, 4, 1, 1>(st, c, rt, M, lg2);
    else stage_hy_scan_t<E, 4, 2, 1>(st, c, rt, M, lg2);
  }
}

// ----------------------------------------------------------------------------- routing
// One wavefront, one token: z fp32 [experts (+ 1: the shared expert's gate)].  Lane s < topk ends up with the s-th choice (ties: the
// lower index) and its share, lane topk with sigmoid of the gate.
// With MK_F_GROUPS (dual kernels): scores are sigmoids, choices are made on score + correction among the experts of the best groups, a
// group's worth being the sum of its two largest; the shares are choice_scale times the scores, the shared expert's is 1.  `scr`: 2 KB
// of LDS of the wavefront.
#if MK_HAVE_DUAL
__device__ __forceinline__ void hy_route_groups(CStage &st, const float *z, int lane, float &w, int &id, float *scr) {
  const int E = st.num_experts, count = st.groups, size = E / count;
  float s[4], p[4];
#pragma unroll
  for (int q = 0; q < 4; q++) {
    const int e = q * 64 + lane, ec = min(e, E - 1);
    const float zv = ldc_f32(z + ec), b = st.choice_bias[ec];
    s[q] = 1.f / (1.f + expf(-zv));
    p[q] = e < E ? s[q] + b : -3.0e38f;
    scr[e] = p[q];
  }
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  if (count > 1) {
    for (int g = lane; g < count; g += 64) {
      float a = -3.0e38f, b = -3.0e38f;
      for (int i = 0; i < size; i++) {
        const float v = scr[g * size + i];
        b = fmaxf(b, fminf(a, v));
        a = fmaxf(a, v);
      }
      scr[256 + g] = size > 1 ? a + b : a;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
    for (int q = 0; q < 4; q++) {
      if (q * 64 >= E) continue;
      const int g = min(q * 64 + lane, E - 1) / size;
      const float mine = scr[256 + g];
      int better = 0;
      for (int i = 0; i < count; i++) {
        const float v = scr[256 + i];
        better += v > mine || (v == mine && i < g);
      }
      if (better >= st.groups_keep) p[q] = -3.0e38f;
    }
  }
  w = 0.f;
  id = 0;
  for (int k = 0; k < st.topk; k++) {
    float bv = p[0];
    int be = lane;
#pragma unroll
    for (int q = 1; q < 4; q++)
      if (p[q] > bv) {
        bv = p[q];
        be = q * 64 + lane;
      }
    wave_argmax(bv, be);
    be = __builtin_amdgcn_readfirstlane(be);
    const float sv = lane_f32(be < 64 ? s[0] : be < 128 ? s[1] : be < 192 ? s[2] : s[3], be & 63);
    if (lane == k) {
      w = sv * st.choice_scale;
      id = be;
    }
#pragma unroll
    for (int q = 0; q < 4; q++)
      if (q * 64 + lane == be) p[q] = -3.4e38f;
  }
  if (lane == st.topk) w = 1.f;
}
#endif
__device__ __forceinline__ void hy_route_wave(CStage &st, const float *z, int lane, float &w, int &id, float *scr) {
#if MK_HAVE_DUAL
  if (st.flags & MK_F_GROUPS) {
    hy_route_groups(st, z, lane, w, id, scr);
    return;
  }
#endif
  const int E = st.num_experts;
  float p[4], mx = -3.0e38f;
#pragma unroll
  for (int q = 0; q < 4; q++) {
    p[q] = q * 64 + lane < E ? ldc_f32(z + q * 64 + lane) : -3.0e38f;
    mx = fmaxf(mx, p[q]);
  }
  const float g = st.w_shared ? ldc_f32(z + E) : 0.f;
  mx = wave_max(mx);
  float sum = 0.f;
#pragma unroll
  for (int q = 0; q < 4; q++) {
    p[q] = q * 64 + lane < E ? expf(p[q] - mx) : 0.f;
    sum += p[q];
  }
  sum = wave_sum(sum);
#pragma unroll
  for (int q = 0; q < 4; q++) p[q] = q * 64 + lane < E ? p[q] / sum : -1.f;
  float tot = 0.f;
  w = 0.f;
  id = 0;
  for (int s = 0; s < st.topk; s++) {
    float bv = p[0];
    int be = lane;
#pragma unroll
    for (int q = 1; q < 4; q++)
      if (p[q] > bv) {
        bv = p[q];
        be = q * 64 + lane;
      }
    wave_argmax(bv, be);
    tot += bv;
    if (lane == s) {
      w = bv;
      id = be;
    }
#pragma unroll
    for (int q = 0; q < 4; q++)
      if (q * 64 + lane == be) p[q] = -1.f;
  }
  w /= tot + 1e-20f;
  if (lane == st.topk) w = 1.f / (1.f + expf(-g));
}
__device__ __forceinline__ void hy_route_store(CStage &st, int t, int lane, float w, int id) {
  if (lane < st.topk) stc_i32(st.ids + (size_t)t * st.topk + lane, id);
  if (lane < st.topk + (st.w_shared ? 1 : 0)) stc_f32((float *)st.slot_w + (size_t)t * st.ld_slot_w + lane, w);
}
// (iterations of several tokens; a single token is routed by the expert stage itself)
__device__ __forceinline__ void stage_hy_route(CStage &st, Ctx &c, int M, char *smem) {
  barrier_wait(c);
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  for (int t = mx_wave_item(c, wave); t < M; t += c.G * MK_WAVES) {
    float w;
    int id;
    hy_route_wave(st, (const float *)st.moe_logits + (size_t)t * st.ld_logits, lane, w, id, (float *)smem + wave * 512);
    hy_route_store(st, t, lane, w, id);
  }
  c.wrote_through = true;
}

// ----------------------------------------------------------------------------- experts
// Weights of an expert are operand tiles (see stage_mx_head_linear); a unit is a pair of 16-row tiles of one expert over all
// tokens that visit it.  Few units: a workgroup per unit, its wavefronts split the reduction; many: a wavefront per unit.  MK_F_SILU: the pair is gate and up of the same 16 outputs, out =
// silu(gate) up.  Expert e < num_experts takes row (token, s) of `in` where s is its place among the token's choices (ld_in_slot 0:
// the token's one row) and writes row (token, s) of `out`; the shared expert has its own sizes and place topk.
// st.n / n_shared: rows of a matrix (gate and up together), st.k / k_shared: reduction length (whole operand rows).
// Units of the shared expert come first: they have the most tokens, and their weights are known before the routing is.
struct HyLists {
  unsigned long long tok[MK_MOE_MAX_EXPERTS];  // tokens that visit the expert
  int active[MK_MOE_MAX_EXPERTS];
  int n_active;
  int pad[3];
  unsigned char place[MK_MOE_MAX_EXPERTS][MK_MAX_TOKENS];
};
static_assert(sizeof(HyLists) <= MK_OUT_OFFSET, "the lists lie below the scratch of the routing and of the reduction");
template <typename E>
__device__ __forceinline__ float hy_glu(E, CStage &st, bool shared, float a, float b) {
#if MK_HAVE_DUAL
  if (st.flags & MK_F_CLAMP_GLU) {
    const float lim = shared ? st.glu_limit_shared : st.glu_limit, g = fminf(a, lim), u = fminf(fmaxf(b, -lim), lim);
    return g * mx_sigmoid(E(), st.glu_beta * g) * (u + st.glu_bias);
  }
#endif
  return hy_silu(E(), a) * b;
}
template <typename E, int MT, bool SPLIT>
__device__ __forceinline__ void hy_expert_unit(CStage &st, const HyLists *ls, bool shared, int e, int pair, unsigned long long toks, int n, int K, int wave, int lane,
                                               const u32x4 *W, const u32x4 (&first)[2][4], f32x4 *red) {
  constexpr int EPC = FxType<E>::EPC, KW = FxType<E>::KW, KB = 4;
  const bool glu = st.flags & MK_F_SILU;
  const int lr = lane & 15, lg = lane >> 4, nks = K / KW, kq = SPLIT ? (nks + MK_WAVES - 1) / MK_WAVES : nks, kb = SPLIT ? min(nks, wave * kq) : 0, ke = min(nks, kb + kq);
  const int cnt = __popcll(toks);
  // lane r gets the r-th token of the list
  const int mine = (toks >> lane) & 1 ? __popcll(toks & ((1ull << lane) - 1ull)) : 63;
  int nth = __builtin_amdgcn_ds_permute(mine << 2, lane);  // (lane 63 may receive several: it is only read when the list holds 64)
  if (cnt == 64) nth = lane;
  int tok[MT], place[MT];
  const E *xr[MT];
#pragma unroll
  for (int m = 0; m < MT; m++) {
    tok[m] = __builtin_amdgcn_ds_bpermute(min(m * 16 + lr, cnt - 1) << 2, nth);
    place[m] = shared ? st.topk : ls->place[e][tok[m]];
    xr[m] = (const E *)st.in + (size_t)tok[m] * st.ld_in + (size_t)place[m] * st.ld_in_slot + lg * EPC;
  }
  f32x4 acc[2][MT];
#pragma unroll
  for (int h = 0; h < 2; h++)
#pragma unroll
    for (int m = 0; m < MT; m++) acc[h][m] = (f32x4){0.f, 0.f, 0.f, 0.f};
  const u32x4 zero = {0u, 0u, 0u, 0u};
  const u32x4 *w0 = W + (size_t)(2 * pair) * nks * 64 + lane, *w1 = w0 + (size_t)nks * 64;
  u32x4 a[2][KB];
#pragma unroll
  for (int h = 0; h < 2; h++)
#pragma unroll
    for (int q = 0; q < KB; q++) a[h][q] = first[h][q];
  for (int k0 = kb; k0 < ke; k0 += KB) {
    u32x4 an[2][KB], b[KB][MT];
#pragma unroll
    for (int q = 0; q < KB; q++)
#pragma unroll
      for (int m = 0; m < MT; m++) b[q][m] = *(const u32x4 *)(xr[m] + (size_t)min(k0 + q, nks - 1) * KW);
#pragma unroll
    for (int q = 0; q < KB; q++) {
      an[0][q] = ldg_stream(w0 + (size_t)min(k0 + KB + q, nks - 1) * 64);
      an[1][q] = ldg_stream(w1 + (size_t)min(k0 + KB + q, nks - 1) * 64);
    }
#pragma unroll
    for (int q = 0; q < KB; q++)
#pragma unroll
      for (int h = 0; h < 2; h++) {
        const u32x4 w = k0 + q < ke ? a[h][q] : zero;
#pragma unroll
        for (int m = 0; m < MT; m++) acc[h][m] = fx_mma_k(E(), w, b[q][m], acc[h][m]);
      }
#pragma unroll
    for (int h = 0; h < 2; h++)
#pragma unroll
      for (int q = 0; q < KB; q++) a[h][q] = an[h][q];
  }
  if constexpr (SPLIT) {
    __syncthreads();
#pragma unroll
    for (int h = 0; h < 2; h++)
#pragma unroll
      for (int m = 0; m < MT; m++) red[((wave * 2 + h) * MT + m) * 64 + lane] = acc[h][m];
    __syncthreads();
  }
  auto total = [&](int h, int m) {
    if constexpr (!SPLIT) return acc[h][m];
    else return red[(h * MT + m) * 64 + lane] + red[((2 + h) * MT + m) * 64 + lane] + red[((4 + h) * MT + m) * 64 + lane] + red[((6 + h) * MT + m) * 64 + lane];
  };
#pragma unroll
  for (int m = 0; m < MT; m++) {
#pragma unroll
    for (int h = 0; h < 2; h++) {
      if ((SPLIT && ((2 * m + h) & (MK_WAVES - 1)) != wave) || m * 16 + lr >= cnt || (glu && h)) continue;
      const f32x4 v = total(h, m);
      float r[4] = {v[0], v[1], v[2], v[3]};
      if (glu) {
        const f32x4 u = total(1, m);
#pragma unroll
        for (int q = 0; q < 4; q++) r[q] = hy_glu(E(), st, shared, r[q], u[q]);
      }
      fx_stc4((E *)st.out + (size_t)tok[m] * st.ld_out + (size_t)place[m] * st.ld_out_slot, (glu ? pair : 2 * pair + h) * 16 + lg * 4, glu ? n / 2 : n, r);
    }
  }
}
template <typename E, int MAXM>
__device__ __forceinline__ void stage_hy_experts(CStage &st, Ctx &c, int M, char *smem) {
  constexpr int KW = FxType<E>::KW;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int Ex = st.num_experts, topk = st.topk;
  const int pairs = (st.n + 31) / 32, pairs_s = st.w_shared ? (st.n_shared + 31) / 32 : 0;
  HyLists *ls = (HyLists *)smem;
  f32x4 *red = (f32x4 *)(smem + MK_MOE_OFFSET);
  struct Unit {
    int e, pair, K, n;
    const u32x4 *W;
  };
  auto unit = [&](int u) {
    Unit a;
    if (u < pairs_s) {
      a = Unit{-1, u, st.k_shared, st.n_shared, (const u32x4 *)st.w_shared};
    } else {
      const int i = (u - pairs_s) / pairs;
      a.pair = (u - pairs_s) - i * pairs;
      a.e = __builtin_amdgcn_readfirstlane(ls->active[i]);
      a.K = st.k;
      a.n = st.n;
      a.W = (const u32x4 *)st.w.seg[0] + (size_t)a.e * pairs * 2 * (st.k / KW) * 64;
    }
    return a;
  };
  u32x4 first[2][4];
  auto load_first = [&](const Unit &a, bool split) {
    const int nks = a.K / KW, kq = (nks + MK_WAVES - 1) / MK_WAVES, kb = split ? min(nks, wave * kq) : 0;
    const u32x4 *w0 = a.W + (size_t)(2 * a.pair) * nks * 64 + lane, *w1 = w0 + (size_t)nks * 64;
#pragma unroll
    for (int q = 0; q < 4; q++) {
      first[0][q] = ldg_stream(w0 + (size_t)min(kb + q, nks - 1) * 64);
      first[1][q] = ldg_stream(w1 + (size_t)min(kb + q, nks - 1) * 64);
    }
  };
  const int u0 = mx_spread(c);
  const bool early = u0 < pairs_s && wave != 0;
  if (early) load_first(unit(u0), true);
  if (tid == 0) __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
  barrier_wait(c);
  // ---- which experts have which tokens
  for (int i = tid; i < Ex; i += MK_THREADS) ls->tok[i] = 0ull;
  __syncthreads();
  if (M == 1 && (st.flags & MK_F_MOE_INLINE_TOPK)) {
    if (wave == MK_WAVES - 1) {
      float w;
      int id;
      hy_route_wave(st, (const float *)st.moe_logits, lane, w, id, (float *)(smem + MK_OUT_OFFSET));
      if (lane < topk) {
        ls->tok[id] = 1ull;
        ls->place[id][0] = (unsigned char)lane;
      }
      if (c.vid == 0) hy_route_store(st, 0, lane, w, id);
    }
  } else {
    for (int i = tid; i < M * topk; i += MK_THREADS) {
      const int t = i / topk, id = ldc_i32(st.ids + i);
      atomicOr(&ls->tok[id], 1ull << t);
      ls->place[id][t] = (unsigned char)(i - t * topk);
    }
  }
  __syncthreads();
  if (wave == 0) {
    int base = 0;
    for (int q = 0; q < Ex; q += 64) {
      const bool has = q + lane < Ex && ls->tok[q + lane] != 0ull;
      const unsigned long long m = __ballot(has);
      if (has) ls->active[base + __popcll(m & ((1ull << lane) - 1ull))] = q + lane;
      base += __popcll(m);
    }
    if (lane == 0) ls->n_active = base;
  }
  __syncthreads();
  const int n_units = pairs_s + __builtin_amdgcn_readfirstlane(ls->n_active) * pairs;
  const unsigned long long all = M >= 64 ? ~0ull : (1ull << M) - 1ull;
  auto walk = [&](auto split, int u, int stride, bool have) {
    constexpr bool SPLIT = decltype(split)::value;
    if (u < n_units && !have) load_first(unit(u), SPLIT);
    for (; u < n_units; u += stride) {
      const Unit a = unit(u);
      u32x4 f[2][4];
#pragma unroll
      for (int h = 0; h < 2; h++)
#pragma unroll
        for (int q = 0; q < 4; q++) f[h][q] = first[h][q];
      if (u + stride < n_units) load_first(unit(u + stride), SPLIT);
      const bool shared = a.e < 0;
      unsigned long long toks = all;
      if (!shared) {
        const unsigned long long t = ls->tok[a.e];
        toks = (unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)t) | ((unsigned long long)(unsigned)__builtin_amdgcn_readfirstlane((int)(t >> 32)) << 32);
      }
      const int cnt = __popcll(toks);
      if constexpr (SPLIT) {  // 16 tokens at a time
        const int rank = (toks >> lane) & 1 ? __popcll(toks & ((1ull << lane) - 1ull)) : -1;
        for (int g = 0; g < cnt; g += 16) hy_expert_unit<E, 1, true>(st, ls, shared, a.e, a.pair, __ballot(rank >= g && rank < g + 16), a.n, a.K, wave, lane, a.W, f, red);
      } else if (cnt <= 16) {
        hy_expert_unit<E, 1, false>(st, ls, shared, a.e, a.pair, toks, a.n, a.K, wave, lane, a.W, f, red);
      } else {
        hy_expert_unit<E, 4, false>(st, ls, shared, a.e, a.pair, toks, a.n, a.K, wave, lane, a.W, f, red);
      }
    }
  };
  if (MAXM == 1 || n_units < 3 * MK_WAVES * c.G) walk(std::true_type{}, u0, c.G, early);
  else if constexpr (MAXM > 1) walk(std::false_type{}, mx_wave_item(c, wave), c.G * MK_WAVES, false);
  c.wrote_through = true;
}
