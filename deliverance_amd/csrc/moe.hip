// Feed-forward layers made of experts: every token's rows go through `top` of `n_experts` small gated
// feed-forwards, and the results are added with weights.
//
//   da_moe_route    from each token's expert ids (read from a table by token id, or given) to a layout in
//                   which every expert's (token, choice) pairs lie together: pairs get slots, an expert's
//                   slots start at a multiple of `tile` rows, so that a tile of rows has one expert; weights
//                   given a pair are also written out a slot
//   da_moe_gated    mid[slot] = act(Wg_e a[row]) * (Wu_e a[row])      (plain kernel, any dtype)
//   da_moe_down     out[slot] = Wd_e mid[slot]                        (plain kernel, 32-bit out)
//   da_moe_combine  y[n] (+)= sum_k weight_k * out[slot(n, k)]        k ascending; a pair without a slot adds weight_k
//                   times the token's input where there are experts that hand it on, and a shared feed-forward's result
//                   joins times a logistic gate
//   da_moe_combine_norm   the same, and the norm of the new stream's rows that the next block starts with
//   da_moe_top, da_moe_choose   from router logits to expert ids and weights; da_moe_choose_route: and to the layout
//
// Everything the grid depends on comes from the step's shape (tokens x top, experts); which tiles are
// used is decided on the device, so a step can be recorded.  A pair's result does not depend on its slot:
// sums over k run in the same order for every row.  Expert weights are stacked: gate | up as
// [n_experts][2 F][K] (gate rows first), down as [n_experts][width][F].
#include "gemm_common.h"

#define MOE_MAX_EXPERTS 1024

struct MoeRouteLds {
  int counts[MOE_MAX_EXPERTS], start[MOE_MAX_EXPERTS], cursor[MOE_MAX_EXPERTS], total;
};

// One workgroup lays the pairs out.  `expert_of(i)`: pair i's expert, or -1.  Every place of row_of_slot and tile_expert is
// written once, so that no barrier has to wait for memory: a pair's slot by the pair, the places behind an expert's last
// pair and the tiles by whoever finds their expert among the starts.
template <class ExpertOf>
__device__ __forceinline__ void moe_lay_out(MoeRouteLds& l, ExpertOf expert_of, int P, int top, int n_experts, int tile,
                                            int* slot_of_pair, int* row_of_slot, int* tile_expert, int P_cap, int T_cap,
                                            const float* pair_weights, float* slot_weight) {
  const int t = threadIdx.x, nt = blockDim.x, lane = t % DA_WAVE;
  for (int e = t; e < n_experts; e += nt) l.counts[e] = l.cursor[e] = 0;
  lds_barrier();
  for (int i = t; i < P; i += nt) {
    const int e = expert_of(i);
    if (e >= 0) atomicAdd(&l.counts[e], 1);
  }
  lds_barrier();
  if (t < DA_WAVE) {                                   // the first wavefront: starts, 64 experts at a time
    int run = 0;
    for (int e0 = 0; e0 < n_experts; e0 += DA_WAVE) {
      const int e = e0 + lane;
      const int own = e < n_experts ? (l.counts[e] + tile - 1) / tile * tile : 0;
      int upto = own;                                  // this expert's slots and those of the ones before it
#pragma unroll
      for (int back = 1; back < DA_WAVE; back *= 2) {
        const int v = __shfl(upto, lane >= back ? lane - back : lane, DA_WAVE);
        if (lane >= back) upto += v;
      }
      if (e < n_experts) l.start[e] = run + upto - own;
      run += __builtin_amdgcn_readlane(upto, DA_WAVE - 1);
    }
    if (t == 0) l.total = run;
  }
  lds_barrier();
  auto owner = [&](int i) -> int {                     // the last expert that starts at or before slot i
    int lo = 0, hi = n_experts - 1;
    while (lo < hi) {
      const int mid = (lo + hi + 1) / 2;
      if (l.start[mid] <= i) lo = mid;
      else hi = mid - 1;
    }
    return lo;
  };
  const int total = l.total;
  for (int i = t; i < P_cap; i += nt) {
    const int e = i < total ? owner(i) : 0;
    if (i >= total || i - l.start[e] >= l.counts[e]) row_of_slot[i] = -1;
  }
  for (int i = t; i < T_cap; i += nt) tile_expert[i] = i * tile < total ? owner(i * tile) : -1;
  for (int i = t; i < P; i += nt) {
    const int e = expert_of(i);
    int slot = -1;
    if (e >= 0) {
      slot = l.start[e] + atomicAdd(&l.cursor[e], 1);
      row_of_slot[slot] = i / top;
      if (pair_weights) slot_weight[slot] = pair_weights[i];      // the pair's weight where its slot's row is
    }
    slot_of_pair[i] = slot;
  }
}

__global__ void __launch_bounds__(1024)
moe_route_kernel(const int* __restrict__ tokens, const int* __restrict__ table, int vocab, const int* __restrict__ ids,
                 int N, int top, int n_experts, int tile, int* __restrict__ slot_of_pair,
                 int* __restrict__ row_of_slot, int* __restrict__ tile_expert, int P_cap, int T_cap,
                 const float* __restrict__ pair_weights, float* __restrict__ slot_weight) {
  __shared__ MoeRouteLds l;
  auto expert_of = [&](int i) -> int {
    int e;
    if (table) {
      const int tok = tokens[i / top];
      e = (tok >= 0 && tok < vocab) ? table[(size_t)tok * top + i % top] : -1;
    } else {
      e = ids[i];
    }
    return (e >= 0 && e < n_experts) ? e : -1;
  };
  moe_lay_out(l, expert_of, N * top, top, n_experts, tile, slot_of_pair, row_of_slot, tile_expert, P_cap, T_cap, pair_weights, slot_weight);
}

extern "C" int da_moe_route(const int* tokens, const int* table, int vocab, const int* ids, int N, int top,
                            int n_experts, int tile, int* slot_of_pair, int* row_of_slot, int* tile_expert, int P_cap,
                            int T_cap, void* stream, const float* pair_weights, float* slot_weight) {
  DA_REQUIRE(N >= 0 && top > 0 && n_experts > 0 && tile > 0, "moe_route: bad sizes");
  DA_REQUIRE(n_experts <= MOE_MAX_EXPERTS, "moe_route: %d experts, %d are taken", n_experts, MOE_MAX_EXPERTS);
  DA_REQUIRE((table != nullptr && tokens != nullptr) != (ids != nullptr), "moe_route: a table with tokens, or expert ids");
  DA_REQUIRE((pair_weights == nullptr) == (slot_weight == nullptr), "moe_route: weights a pair need a place a slot");
  DA_REQUIRE(T_cap >= da_ceil_div((long)N * top, tile) + n_experts && P_cap >= T_cap * tile,
             "moe_route: the slot space (%d rows, %d tiles) is too small for %d pairs", P_cap, T_cap, N * top);
  if (N == 0) return 0;
  hipLaunchKernelGGL(moe_route_kernel, dim3(1), dim3(1024), 0, (hipStream_t)stream, tokens, table, vocab, ids, N, top,
                     n_experts, tile, slot_of_pair, row_of_slot, tile_expert, P_cap, T_cap, pair_weights, slot_weight);
  DA_CHECK_LAUNCH("moe_route");
  return 0;
}

// ---- plain grouped products: tiles of 64 x 64, sums in two levels as the plain product has them ------------
#define MT 64
#define MBK 16
#define MCHUNK 8

// MOE_GATED: two products (gate and up rows of the expert's stacked matrix), out = act(g) * u in T; MOE_UP: one
// product, out = act(.) in T; MOE_DOWN: one product, 32-bit out.  The first two gather: row r of the tile is
// a[row_of_slot[slot]] (times slot_scale[slot] when given: the sums are scaled, which is the same number),
// MOE_DOWN reads a[slot].
#define MOE_DOWN 0
#define MOE_GATED 1
#define MOE_UP 2
template <typename T, int MODE>
__global__ void __launch_bounds__(256)
moe_product_ref_kernel(const T* __restrict__ a, int lda, const int* __restrict__ row_of_slot,
                       const int* __restrict__ tile_expert, const T* __restrict__ w, void* __restrict__ out, int ldo,
                       int K, int F, int act, const float* __restrict__ slot_scale, float limit) {
  constexpr bool GATED = MODE == MOE_GATED, GATHER = MODE != MOE_DOWN;
  const int e = tile_expert[blockIdx.y];
  if (e < 0) return;
  __shared__ float As[MBK][MT + 4];
  __shared__ float Ws[GATED ? 2 : 1][MBK][MT + 4];
  __shared__ int srow[MT];
  const int t = threadIdx.x;
  const int tx = t % 16, ty = t / 16;
  const int m0 = blockIdx.y * MT, n0 = blockIdx.x * MT;
  const int lrow = t / 4, lk = (t % 4) * 4;
  if (t < MT) srow[t] = row_of_slot[m0 + t];
  __syncthreads();
  const T* wg = w + (size_t)e * (GATED ? 2 : 1) * F * K;
  const T* wu = wg + (size_t)F * K;
  float acc[GATED ? 2 : 1][4][4], part[GATED ? 2 : 1][4][4];
#pragma unroll
  for (int g = 0; g < (GATED ? 2 : 1); ++g)
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[g][i][j] = part[g][i][j] = 0.f;
  const int arow = GATHER ? srow[lrow] : (srow[lrow] >= 0 ? m0 + lrow : -1);
  int slab = 0;
  for (int k0 = 0; k0 < K; k0 += MBK) {
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int k = k0 + lk + x;
      const int wn = n0 + lrow;
      As[lk + x][lrow] = (arow >= 0 && k < K) ? to_f32(a[(size_t)arow * lda + k]) : 0.f;
      Ws[0][lk + x][lrow] = (wn < F && k < K) ? to_f32(wg[(size_t)wn * K + k]) : 0.f;
      if (GATED) Ws[1][lk + x][lrow] = (wn < F && k < K) ? to_f32(wu[(size_t)wn * K + k]) : 0.f;
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < MBK; ++k) {
      float av[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) av[i] = As[k][ty * 4 + i];
#pragma unroll
      for (int g = 0; g < (GATED ? 2 : 1); ++g) {
        float wv[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) wv[j] = Ws[g][k][tx * 4 + j];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int j = 0; j < 4; ++j) part[g][i][j] = fmaf(av[i], wv[j], part[g][i][j]);
      }
    }
    if (++slab == MCHUNK) {
      slab = 0;
#pragma unroll
      for (int g = 0; g < (GATED ? 2 : 1); ++g)
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            acc[g][i][j] += part[g][i][j];
            part[g][i][j] = 0.f;
          }
    }
    __syncthreads();
  }
#pragma unroll
  for (int g = 0; g < (GATED ? 2 : 1); ++g)
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[g][i][j] += part[g][i][j];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = ty * 4 + i;
    if (srow[r] < 0) continue;
    const float sc = (GATHER && slot_scale) ? slot_scale[m0 + r] : 1.0f;      // the row of a times its weight
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + tx * 4 + j;
      if (n >= F) continue;
      const size_t o = (size_t)(m0 + r) * ldo + n;
      if (GATED) {
        from_f32(&((T*)out)[o], gated_mid<DTypeOf<T>::value == DA_BF16>(sc * acc[0][i][j], sc * acc[1][i][j], act, limit));
      } else if (MODE == MOE_UP) {
        from_f32(&((T*)out)[o], DTypeOf<T>::value == DA_BF16 ? apply_act_bf16(sc * acc[0][i][j], act) : apply_act(sc * acc[0][i][j], act));
      } else {
        ((float*)out)[o] = acc[0][i][j];
      }
    }
  }
}

extern "C" int da_moe_gated_ref(const void* a, int lda, int dtype, const int* row_of_slot, const int* tile_expert,
                                const void* w, void* mid, int ldm, int T_cap, int K, int F, int act, float limit,
                                void* stream) {
  DA_REQUIRE(T_cap >= 0 && K > 0 && F > 0 && lda >= K && ldm >= F, "moe_gated_ref: bad sizes");
  DA_REQUIRE(act != DA_ACT_GLU_CAPPED || limit > 0.f, "moe_gated_ref: the capped form needs a positive limit");
  DA_REQUIRE(act >= DA_ACT_NONE && act <= DA_ACT_LAST, "moe_gated_ref: unknown activation %d", act);
  if (T_cap == 0) return 0;
  dim3 grid(da_ceil_div(F, MT), T_cap);
  if (dtype == DA_BF16)
    hipLaunchKernelGGL((moe_product_ref_kernel<bf16_t, MOE_GATED>), grid, dim3(256), 0, (hipStream_t)stream, (const bf16_t*)a,
                       lda, row_of_slot, tile_expert, (const bf16_t*)w, mid, ldm, K, F, act, nullptr, limit);
  else
    hipLaunchKernelGGL((moe_product_ref_kernel<float, MOE_GATED>), grid, dim3(256), 0, (hipStream_t)stream, (const float*)a,
                       lda, row_of_slot, tile_expert, (const float*)w, mid, ldm, K, F, act, nullptr, limit);
  DA_CHECK_LAUNCH("moe_gated_ref");
  return 0;
}

extern "C" int da_moe_down_ref(const void* mid, int ldm, int dtype, const int* row_of_slot, const int* tile_expert,
                               const void* w, float* out, int ldo, int T_cap, int F, int width, void* stream) {
  DA_REQUIRE(T_cap >= 0 && F > 0 && width > 0 && ldm >= F && ldo >= width, "moe_down_ref: bad sizes");
  if (T_cap == 0) return 0;
  dim3 grid(da_ceil_div(width, MT), T_cap);
  if (dtype == DA_BF16)
    hipLaunchKernelGGL((moe_product_ref_kernel<bf16_t, MOE_DOWN>), grid, dim3(256), 0, (hipStream_t)stream,
                       (const bf16_t*)mid, ldm, row_of_slot, tile_expert, (const bf16_t*)w, out, ldo, F, width, 0, nullptr, 0.f);
  else
    hipLaunchKernelGGL((moe_product_ref_kernel<float, MOE_DOWN>), grid, dim3(256), 0, (hipStream_t)stream,
                       (const float*)mid, ldm, row_of_slot, tile_expert, (const float*)w, out, ldo, F, width, 0, nullptr, 0.f);
  DA_CHECK_LAUNCH("moe_down_ref");
  return 0;
}

// mid[slot] = act(scale[slot] * (W_e a[row_of_slot[slot]])): the first product of experts without a gate; w: [experts, F, K]
extern "C" int da_moe_up_ref(const void* a, int lda, int dtype, const int* row_of_slot, const int* tile_expert,
                             const void* w, const float* slot_scale, void* mid, int ldm, int T_cap, int K, int F, int act,
                             void* stream) {
  DA_REQUIRE(T_cap >= 0 && K > 0 && F > 0 && lda >= K && ldm >= F, "moe_up_ref: bad sizes");
  DA_REQUIRE(act >= DA_ACT_NONE && act <= DA_ACT_LAST, "moe_up_ref: unknown activation %d", act);
  if (T_cap == 0) return 0;
  dim3 grid(da_ceil_div(F, MT), T_cap);
  if (dtype == DA_BF16)
    hipLaunchKernelGGL((moe_product_ref_kernel<bf16_t, MOE_UP>), grid, dim3(256), 0, (hipStream_t)stream, (const bf16_t*)a,
                       lda, row_of_slot, tile_expert, (const bf16_t*)w, mid, ldm, K, F, act, slot_scale, 0.f);
  else
    hipLaunchKernelGGL((moe_product_ref_kernel<float, MOE_UP>), grid, dim3(256), 0, (hipStream_t)stream, (const float*)a,
                       lda, row_of_slot, tile_expert, (const float*)w, mid, ldm, K, F, act, slot_scale, 0.f);
  DA_CHECK_LAUNCH("moe_up_ref");
  return 0;
}

// The router's choice from 32-bit logits z (+ bias, when given): every token's `top` largest (the lower index wins a
// tie), ids[n, k] and weights[n, k] in descending order.  mode 0: the weights are logistic(z) (`renorm`: divided by
// their sum); mode 1: the softmax over the chosen logits only.
__global__ void moe_top_kernel(const float* __restrict__ z, int ldz, const void* __restrict__ bias, int bias_dtype, int N,
                               int E, int top, int mode, int renorm, int* __restrict__ ids, float* __restrict__ weights) {
  const int n = blockIdx.x * blockDim.x + threadIdx.x;
  if (n >= N) return;
  const float* row = z + (size_t)n * ldz;
  float sum = 0.f, first = 0.f;
  for (int k = 0; k < top; ++k) {
    int best = -1;
    float bz = -INFINITY;
    for (int e = 0; e < E; ++e) {
      const float v = row[e] + (bias ? load_param(bias, bias_dtype, e) : 0.f);
      bool taken = false;
      for (int j = 0; j < k; ++j) taken |= ids[(size_t)n * top + j] == e;
      if (!taken && (best < 0 || v > bz)) { best = e; bz = v; }
    }
    if (k == 0) first = bz;
    const float sc = mode == 1 ? expf(bz - first) : 1.0f / (1.0f + expf(-bz));
    ids[(size_t)n * top + k] = best;
    weights[(size_t)n * top + k] = sc;
    sum += sc;
  }
  if (renorm || mode == 1)
    for (int k = 0; k < top; ++k) weights[(size_t)n * top + k] /= sum;
}

extern "C" int da_moe_top(const float* z, int ldz, const void* bias, int bias_dtype, int N, int E, int top, int mode,
                          int renorm, int* ids, float* weights, void* stream) {
  DA_REQUIRE(N >= 0 && E > 0 && top > 0 && top <= E && ldz >= E, "moe_top: bad sizes");
  DA_REQUIRE(mode == 0 || mode == 1, "moe_top: mode %d (0: logistic scores, 1: softmax over the chosen)", mode);
  if (N == 0) return 0;
  hipLaunchKernelGGL(moe_top_kernel, dim3(da_ceil_div(N, 64)), dim3(64), 0, (hipStream_t)stream, z, ldz, bias, bias_dtype, N,
                     E, top, mode, renorm, ids, weights);
  DA_CHECK_LAUNCH("moe_top");
  return 0;
}

extern "C" int da_moe_top_logistic(const float* z, int ldz, int N, int E, int top, int renorm, int* ids, float* weights,
                                   void* stream) {
  return da_moe_top(z, ldz, nullptr, 0, N, E, top, 0, renorm, ids, weights, stream);
}

// The choice by a softmax over all E outputs: s = softmax(z), c = s + correction; the `top` largest c are chosen (the lower
// index wins a tie), with s over the chosen ones' sum (+ 1e-20) as weights.  groups > 0: the outputs are so many equal runs
// of neighbours, a run counts as its largest c, and only entries of the `keep` best runs can be chosen (the lower run wins
// a tie).  A wavefront a token, an output every 64th a lane; c and the runs' largest wait in LDS.
// One wavefront works on one token; `c`, `sc`, `gm`: its LDS, E entries each (choice scores, softmax scores, the runs'
// largest).  `give(k, output, score)` receives the choices, lane 0 only; returns the sum of their scores.
template <class Give>
__device__ __forceinline__ float moe_choose_token(const float* __restrict__ row, const float* __restrict__ correction, int E, int top,
                                                  int groups, int keep, float* c, float* sc, float* gm, int lane, Give give) {
  auto wave_fence = [] {                               // LDS of this wavefront only
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
  };
  const float corr0 = correction[lane < E ? lane : 0];       // (asked for ahead of the sums)
  float m = -INFINITY;
  for (int e = lane; e < E; e += DA_WAVE) m = fmaxf(m, row[e]);
  m = wave_max(m);
  float sum = 0.f;
  for (int e = lane; e < E; e += DA_WAVE) {
    const float v = expf(row[e] - m);
    sc[e] = v;
    sum += v;
  }
  sum = wave_sum(sum);
  for (int e = lane; e < E; e += DA_WAVE) {
    const float v = sc[e] / sum;
    sc[e] = v;
    c[e] = v + (e < DA_WAVE ? corr0 : correction[e]);
  }
  wave_fence();
  if (groups > 0) {
    const int size = E / groups;
    for (int q = lane; q < groups; q += DA_WAVE) {
      float v = -INFINITY;
      for (int e = 0; e < size; ++e) v = fmaxf(v, c[q * size + e]);
      gm[q] = v;
    }
    wave_fence();
    for (int q = lane; q < groups; q += DA_WAVE) {
      int ahead = 0;                                   // runs that come before this one
      for (int k = 0; k < groups; ++k) ahead += gm[k] > gm[q] || (gm[k] == gm[q] && k < q);
      if (ahead >= keep)
        for (int e = 0; e < size; ++e) c[q * size + e] = -INFINITY;
    }
    wave_fence();
  }
  float chosen = 0.f;
  auto better = [](float a, int ai, float b, int bi) { return a > b || (a == b && ai < bi); };
  for (int k = 0; k < top; ++k) {
    float bv = -INFINITY;
    int be = lane < E ? lane : E - 1;
    for (int e = lane; e < E; e += DA_WAVE)
      if (better(c[e], e, bv, be)) { bv = c[e]; be = e; }
    wave_best(bv, be, better);
    const float s = sc[be];
    chosen += s;
    if (lane == 0) {
      give(k, be, s);
      c[be] = -INFINITY;                               // taken
    }
    wave_fence();
  }
  return chosen;
}

// The same for at most 64 outputs: an output a lane, everything in registers.
template <class Give>
__device__ __forceinline__ float moe_choose_token64(const float* __restrict__ row, float corr, int E, int top, int groups, int keep,
                                                    int lane, Give give) {
  const bool in = lane < E;                            // corr: this lane's output's
  const float z = in ? row[lane] : -INFINITY;
  const float m = wave_max(z);                         // (every lane takes part in what goes across lanes)
  const float ex = in ? expf(z - m) : 0.f;
  const float s = ex / wave_sum(ex);
  float c = in ? s + corr : -INFINITY;
  if (groups > 0) {
    const int size = E / groups, mine = (in ? lane : 0) / size;
    float best = -INFINITY;                            // of this lane's run
    for (int e = 0; e < size; ++e) best = fmaxf(best, __shfl(c, mine * size + e, DA_WAVE));
    int ahead = 0;                                     // runs that come before it
    for (int k = 0; k < groups; ++k) {
      const float other = __shfl(best, k * size, DA_WAVE);
      ahead += other > best || (other == best && k < mine);
    }
    if (ahead >= keep) c = -INFINITY;
  }
  float chosen = 0.f;
  auto better = [](float a, int ai, float b, int bi) { return a > b || (a == b && ai < bi); };
  for (int k = 0; k < top; ++k) {
    float bv = c;
    int be = in ? lane : E - 1;
    wave_best(bv, be, better);
    const float sb = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, s), be));
    chosen += sb;
    if (lane == 0) give(k, be, sb);
    if (lane == be) c = -INFINITY;                     // taken
  }
  return chosen;
}

// (EC: outputs that LDS has room for.)
#define MC_WAVES 4
template <int EC>
__global__ void __launch_bounds__(MC_WAVES * DA_WAVE)
moe_choose_kernel(const float* __restrict__ z, int ldz, const float* __restrict__ correction, int N, int E, int top, int groups,
                  int keep, int extra, int n_experts, int* __restrict__ ids, float* __restrict__ weights) {
  __shared__ float mc_lds[EC > 64 ? MC_WAVES : 1][3][EC > 64 ? EC : 1];
  const int lane = threadIdx.x % DA_WAVE, wave = threadIdx.x / DA_WAVE;
  const int n = blockIdx.x * MC_WAVES + wave;
  if (n >= N) return;                                  // (wavefronts do not wait for one another)
  const float* row = z + (size_t)n * ldz;
  const float gate = extra ? row[E] : 0.f;
  int* const id = ids + (size_t)n * (top + extra);
  float* const w = weights + (size_t)n * (top + extra);
  float sum;
  auto give = [&](int k, int e, float s) {
    id[k] = e < n_experts ? e : e + extra;
    w[k] = s;
  };
  if (EC <= 64) sum = moe_choose_token64(row, correction[lane < E ? lane : 0], E, top, groups, keep, lane, give);
  else sum = moe_choose_token(row, correction, E, top, groups, keep, mc_lds[EC > 64 ? wave : 0][0], mc_lds[EC > 64 ? wave : 0][1],
                              mc_lds[EC > 64 ? wave : 0][2], lane, give);
  if (lane == 0)
    for (int k = 0; k < top; ++k) w[k] /= sum + 1e-20f;
  for (int k = lane; k < extra; k += DA_WAVE) {
    id[top + k] = n_experts + k;
    w[top + k] = 1.f / (1.f + expf(-gate));
  }
}

// ids[n] and weights[n]: `top` choices (outputs from n_experts on, experts that hand their input on, become ids from n_experts
// + extra on), then the `extra` further experts n_experts .., which every token uses with the weight logistic(z[n, E]).
extern "C" int da_moe_choose(const float* z, int ldz, const float* correction, int N, int E, int top, int groups, int keep,
                             int extra, int n_experts, int* ids, float* weights, void* stream) {
  DA_REQUIRE(N >= 0 && E > 0 && E <= MOE_MAX_EXPERTS && top > 0 && top <= E && extra >= 0 && n_experts > 0 && n_experts <= E &&
             ldz >= E + (extra > 0) && correction, "moe_choose: bad sizes");
  DA_REQUIRE(groups == 0 || (groups > 0 && E % groups == 0 && keep > 0 && keep <= groups && top <= E / groups * keep),
             "moe_choose: top %d of %d outputs in %d groups of which %d are kept", top, E, groups, keep);
  if (N == 0) return 0;
#define MC_GO(EC)                                                                                                            \
  hipLaunchKernelGGL((moe_choose_kernel<EC>), dim3(da_ceil_div(N, MC_WAVES)), dim3(MC_WAVES * DA_WAVE), 0, (hipStream_t)stream, \
                     z, ldz, correction, N, E, top, groups, keep, extra, n_experts, ids, weights)
  if (E <= 64) MC_GO(64);
  else if (E <= 256) MC_GO(256);
  else MC_GO(MOE_MAX_EXPERTS);
#undef MC_GO
  DA_CHECK_LAUNCH("moe_choose");
  return 0;
}

// The products of all tokens' inputs with one row of a router, by one wavefront: a lane holds every 64th run of 8 entries,
// the row and MR_TOKENS inputs are asked for at once, and a sum is added up across the lanes in a fixed order.
#define MR_TOKENS 8
template <class Give>
__device__ __forceinline__ void moe_router_row(const bf16_t* __restrict__ h, int ldh, int N, const bf16_t* __restrict__ row, int K,
                                               int lane, Give give) {
  for (int n0 = 0; n0 < N; n0 += MR_TOKENS) {
    float acc[MR_TOKENS];
#pragma unroll
    for (int j = 0; j < MR_TOKENS; ++j) acc[j] = 0.f;
    for (int k = lane * 8; k < K; k += 8 * DA_WAVE) {
      uint4 hv[MR_TOKENS];
      const uint4 wv = load16(row + k);
#pragma unroll
      for (int j = 0; j < MR_TOKENS; ++j) hv[j] = load16(h + (size_t)(n0 + j < N ? n0 + j : N - 1) * ldh + k);
      const uint32_t b[4] = {wv.x, wv.y, wv.z, wv.w};
#pragma unroll
      for (int j = 0; j < MR_TOKENS; ++j) {
        const uint32_t a[4] = {hv[j].x, hv[j].y, hv[j].z, hv[j].w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          acc[j] = fmaf(__uint_as_float(a[e] << 16), __uint_as_float(b[e] << 16), acc[j]);
          acc[j] = fmaf(__uint_as_float(a[e] & 0xffff0000u), __uint_as_float(b[e] & 0xffff0000u), acc[j]);
        }
      }
    }
#pragma unroll
    for (int j = 0; j < MR_TOKENS; ++j) {
      const float v = wave_sum(acc[j]);
      if (lane == 0 && n0 + j < N) give(n0 + j, v);
    }
  }
}

// The smallest steps: the router's product (h, router [E (+ 1)][K] in bfloat16, sums in 32-bit; or z holds its results), the
// choice, and the pairs' layout in one launch.  ids and weights as da_moe_choose has them.
#define MCR_WAVES 16
#define MCR_MAX_OUTPUTS 64
#define MCR_MAX_TOKENS 16
#define MCR_MAX_PAIRS 1024
#define MCR_MAX_ROUTER_STEPS 8        // round trips to memory of a wavefront
__global__ void __launch_bounds__(MCR_WAVES * DA_WAVE)
moe_choose_route_kernel(const bf16_t* __restrict__ h, int ldh, const bf16_t* __restrict__ router, int K,
                        const float* __restrict__ z, int ldz, const float* __restrict__ correction, int N, int E, int top, int groups,
                        int keep, int extra, int n_experts, int tile, int* __restrict__ ids, float* __restrict__ weights,
                        int* __restrict__ slot_of_pair, int* __restrict__ row_of_slot, int* __restrict__ tile_expert, int P_cap,
                        int T_cap) {
  __shared__ float logits[MCR_MAX_TOKENS][MCR_MAX_OUTPUTS + 1];
  __shared__ MoeRouteLds l;
  __shared__ int pair[MCR_MAX_PAIRS];
  __shared__ float score[MCR_MAX_PAIRS];
  const int lane = threadIdx.x % DA_WAVE, wave = threadIdx.x / DA_WAVE, each = top + extra;
  const float corr = correction[lane < E ? lane : 0];  // (asked for first)
  if (h) {                                             // the logits are made here
    for (int r = wave; r < E + (extra > 0); r += MCR_WAVES)
      moe_router_row(h, ldh, N, router + (size_t)r * K, K, lane, [&](int n, float v) { logits[n][r] = v; });
    lds_barrier();
  }
  const int n = wave;                                  // a token a wavefront
  if (n < N) {
    int* const pr = pair + n * each;
    float* const sc = score + n * each;
    const float* row = h ? logits[n] : z + (size_t)n * ldz;
    const float gate = extra ? row[E] : 0.f;
    const float sum = moe_choose_token64(row, corr, E, top, groups, keep, lane, [&](int k, int e, float s) {
      pr[k] = e < n_experts ? e : e + extra;
      sc[k] = s;
    });
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
    for (int k = lane; k < each; k += DA_WAVE) {
      const int e = k < top ? pr[k] : n_experts + (k - top);
      if (k >= top) pr[k] = e;
      ids[(size_t)n * each + k] = e;
      weights[(size_t)n * each + k] = k < top ? sc[k] / (sum + 1e-20f) : 1.f / (1.f + expf(-gate));
    }
  }
  lds_barrier();
  moe_lay_out(l, [&](int i) -> int { const int e = pair[i]; return e < n_experts + extra ? e : -1; }, N * each, each, n_experts + extra, tile,
              slot_of_pair, row_of_slot, tile_expert, P_cap, T_cap, nullptr, nullptr);
}

extern "C" int da_moe_choose_route_takes(int N, int E, int top, int extra, int n_experts) {
  return N <= MCR_MAX_TOKENS && E <= MCR_MAX_OUTPUTS && (long)N * (top + extra) <= MCR_MAX_PAIRS && n_experts + extra <= MOE_MAX_EXPERTS;
}

// 1 when it pays to make the logits there too
extern "C" int da_moe_choose_route_takes_router(int N, int rows, int K) {
  return N > 0 && N <= MCR_MAX_TOKENS && rows <= MCR_MAX_OUTPUTS + 1 && K % 8 == 0 &&
         (long)da_ceil_div(rows, MCR_WAVES) * da_ceil_div(N, MR_TOKENS) * da_ceil_div(K, 8 * DA_WAVE) <= MCR_MAX_ROUTER_STEPS;
}

extern "C" int da_moe_choose_route(const void* h, int ldh, const void* router, int K, const float* z, int ldz, const float* correction, int N, int E, int top, int groups, int keep,
                                   int extra, int n_experts, int tile, int* ids, float* weights, int* slot_of_pair, int* row_of_slot,
                                   int* tile_expert, int P_cap, int T_cap, void* stream) {
  DA_REQUIRE(N >= 0 && E > 0 && top > 0 && top <= E && extra >= 0 && n_experts > 0 && n_experts <= E && tile > 0 &&
             correction && (h || (z && ldz >= E + (extra > 0))), "moe_choose_route: bad sizes");
  DA_REQUIRE(!h || (router && N <= MCR_MAX_TOKENS && K > 0 && K % 8 == 0 && ldh >= K && ldh % 8 == 0 && ((uintptr_t)h | (uintptr_t)router) % 16 == 0),
             "moe_choose_route: the router's operands (rows of multiples of 8 entries, 16-byte aligned)");
  DA_REQUIRE(da_moe_choose_route_takes(N, E, top, extra, n_experts), "moe_choose_route: %d tokens with %d of %d outputs are not taken", N, top + extra, E);
  DA_REQUIRE(groups == 0 || (groups > 0 && E % groups == 0 && keep > 0 && keep <= groups && top <= E / groups * keep),
             "moe_choose_route: top %d of %d outputs in %d groups of which %d are kept", top, E, groups, keep);
  DA_REQUIRE(T_cap >= da_ceil_div((long)N * (top + extra), tile) + n_experts + extra && P_cap >= T_cap * tile,
             "moe_choose_route: the slot space (%d rows, %d tiles) is too small", P_cap, T_cap);
  if (N == 0) return 0;
  hipLaunchKernelGGL(moe_choose_route_kernel, dim3(1), dim3(MCR_WAVES * DA_WAVE), 0, (hipStream_t)stream, (const bf16_t*)h, ldh,
                     (const bf16_t*)router, K, z, ldz, correction, N, E, top, groups, keep, extra, n_experts, tile, ids, weights, slot_of_pair, row_of_slot, tile_expert, P_cap, T_cap);
  DA_CHECK_LAUNCH("moe_choose_route");
  return 0;
}

// slot_weight[slot_of_pair[i]] = weights[i]: a pair's weight where its slot's row is
__global__ void moe_slot_weights_kernel(const int* __restrict__ slot_of_pair, const float* __restrict__ weights, int P,
                                        float* __restrict__ slot_weight) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= P) return;
  const int slot = slot_of_pair[i];
  if (slot >= 0) slot_weight[slot] = weights[i];
}

extern "C" int da_moe_slot_weights(const int* slot_of_pair, const float* weights, int P, float* slot_weight, void* stream) {
  DA_REQUIRE(P >= 0, "moe_slot_weights: bad size");
  if (P == 0) return 0;
  hipLaunchKernelGGL(moe_slot_weights_kernel, dim3(da_ceil_div(P, 256)), dim3(256), 0, (hipStream_t)stream, slot_of_pair,
                     weights, P, slot_weight);
  DA_CHECK_LAUNCH("moe_slot_weights");
  return 0;
}

// y[n] (+)= sum_k weight(n, k) * out[slot_of_pair[n * top + k]]; weights: per pair, or one for all.  h (optional): a pair
// without a slot adds weight * h[n], an expert that hands its input on.  shared (optional): + logistic(gate[n]) * shared[n].
template <typename T>
__global__ void moe_combine_kernel(const float* __restrict__ out, int ldo, const int* __restrict__ slot_of_pair,
                                   const float* __restrict__ weights, float uniform, int top, float* __restrict__ y,
                                   int ldy, int N, int width, int accumulate, const T* __restrict__ h, int ldh,
                                   const float* __restrict__ shared, int lds, const float* __restrict__ gate, int ldg) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= (long)N * width) return;
  const int n = (int)(i / width), c = (int)(i % width);
  float s = 0.f;
  for (int k = 0; k < top; ++k) {
    const int slot = slot_of_pair[n * top + k];
    if (slot >= 0) s += (weights ? weights[n * top + k] : uniform) * out[(size_t)slot * ldo + c];
    else if (h) s += (weights ? weights[n * top + k] : uniform) * to_f32(h[(size_t)n * ldh + c]);
  }
  if (shared) s += shared[(size_t)n * lds + c] / (1.f + expf(-gate[(size_t)n * ldg]));
  float* dst = y + (size_t)n * ldy + c;
  *dst = accumulate ? *dst + s : s;
}

extern "C" int da_moe_combine(const float* out, int ldo, const int* slot_of_pair, const float* weights, float uniform,
                              int top, float* y, int ldy, int N, int width, int accumulate, const void* h, int h_dtype, int ldh,
                              const float* shared, int lds, const float* gate, int ldg, void* stream) {
  DA_REQUIRE(N >= 0 && width > 0 && top > 0 && ldo >= width && ldy >= width, "moe_combine: bad sizes");
  DA_REQUIRE((!h || ldh >= width) && (!shared || (lds >= width && gate && ldg > 0)), "moe_combine: the input's or the shared result's rows");
  if (N == 0) return 0;
  const dim3 grid(da_ceil_div((long)N * width, 256));
  if (h && h_dtype == DA_BF16)
    hipLaunchKernelGGL(moe_combine_kernel<bf16_t>, grid, dim3(256), 0, (hipStream_t)stream, out, ldo, slot_of_pair, weights,
                       uniform, top, y, ldy, N, width, accumulate, (const bf16_t*)h, ldh, shared, lds, gate, ldg);
  else
    hipLaunchKernelGGL(moe_combine_kernel<float>, grid, dim3(256), 0, (hipStream_t)stream, out, ldo, slot_of_pair, weights,
                       uniform, top, y, ldy, N, width, accumulate, (const float*)h, ldh, shared, lds, gate, ldg);
  DA_CHECK_LAUNCH("moe_combine");
  return 0;
}

// The same for a step's rows one by one, with what follows the feed-forward: the stream's row takes the pairs' sum (and
// `add` [N][width], `vec` [width], when the stream is changed before the next block), and the next block's norm of the new
// row leaves in h_next.  centre: (x - mean) / sqrt(var + eps) * gain (+ bias); else x / sqrt(mean x^2 + eps) * (offset +
// gain).  A wavefront owns a row, VPL float4 a lane (width a multiple of 4, at most 256 * VPL); all in 32-bit.
template <int VPL> struct McnPairs { static const int value = VPL <= 4 ? 4 : (VPL <= 8 ? 2 : 1); };
struct CombineNorm {
  const float* out; int ldo;
  const int* slot_of_pair;
  const float* weights; float uniform; int top;
  float* y;                        // the stream [N][width]
  const void* h; int ldh;          // the input that pairs without a slot hand on, or null
  const float* shared; int lds;    // with a logistic gate a row, or null
  const float* gate; int ldg;
  const float* add; const float* vec;
  const void* gain; int gain_dtype;
  const void* bias; int bias_dtype;
  float offset, eps; int centre;
  void* h_next;                    // [N][width], h's dtype
  int N, width, accumulate;
};

__device__ __forceinline__ float4 mcn_load4(const float* p) { return *(const float4*)p; }
__device__ __forceinline__ float4 mcn_load4(const bf16_t* p) {
  const uint2 u = *(const uint2*)p;
  return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16), __uint_as_float(u.y & 0xffff0000u));
}
__device__ __forceinline__ float4 mcn_param4(const void* p, int dtype, int i) {
  return dtype == DA_BF16 ? mcn_load4((const bf16_t*)p + i) : mcn_load4((const float*)p + i);
}
__device__ __forceinline__ float4 mcn_fma(float w, float4 a, float4 s) {
  return make_float4(fmaf(w, a.x, s.x), fmaf(w, a.y, s.y), fmaf(w, a.z, s.z), fmaf(w, a.w, s.w));
}

template <typename T, int VPL>
__global__ void __launch_bounds__(4 * DA_WAVE)
moe_combine_norm_kernel(CombineNorm p) {
  const int lane = threadIdx.x % DA_WAVE;
  const int n = blockIdx.x * (blockDim.x / DA_WAVE) + threadIdx.x / DA_WAVE;
  if (n >= p.N) return;
  const int E = p.width;
  constexpr int PAIRS = McnPairs<VPL>::value;
  // Everything whose place is known is asked for at once: the stream's row, the norm's parameters, the first pairs' slots
  // and weights, the input that is handed on, the shared result; then PAIRS pairs' rows at a time (a pair without a
  // slot reads row 0 and counts as nothing: looked at afterwards, a load under a condition would be waited for on the spot).
  float4 x[VPL], g[VPL], b[VPL], s[VPL], hv[VPL], sv[VPL];
  int at[VPL], slot[PAIRS];
  float w[PAIRS];
  auto ask = [&](int k0) {
#pragma unroll
    for (int k = 0; k < PAIRS; ++k) {
      const size_t i = (size_t)n * p.top + (k0 + k < p.top ? k0 + k : 0);
      slot[k] = p.slot_of_pair[i];
      w[k] = p.weights ? p.weights[i] : p.uniform;
    }
  };
  ask(0);
#pragma unroll
  for (int i = 0; i < VPL; ++i) {
    const int c = (lane + i * DA_WAVE) * 4;
    at[i] = c < E ? c : 0;
    s[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    x[i] = mcn_load4(p.y + (size_t)n * E + at[i]);
    g[i] = mcn_param4(p.gain, p.gain_dtype, at[i]);
    b[i] = p.bias ? mcn_param4(p.bias, p.bias_dtype, at[i]) : make_float4(0.f, 0.f, 0.f, 0.f);
    if (p.h) hv[i] = mcn_load4((const T*)p.h + (size_t)n * p.ldh + at[i]);
    if (p.shared) sv[i] = mcn_load4(p.shared + (size_t)n * p.lds + at[i]);
  }
  const float gate = p.shared ? p.gate[(size_t)n * p.ldg] : 0.f;
  float handed_on = 0.f;
  for (int k0 = 0; k0 < p.top; k0 += PAIRS) {
    if (k0) ask(k0);
    float4 v[PAIRS][VPL];
#pragma unroll
    for (int k = 0; k < PAIRS; ++k)
#pragma unroll
      for (int i = 0; i < VPL; ++i) v[k][i] = mcn_load4(p.out + (size_t)(slot[k] >= 0 ? slot[k] : 0) * p.ldo + at[i]);
#pragma unroll
    for (int k = 0; k < PAIRS; ++k) {
      if (k0 + k >= p.top) continue;
      if (slot[k] >= 0) {
#pragma unroll
        for (int i = 0; i < VPL; ++i) s[i] = mcn_fma(w[k], v[k][i], s[i]);
      } else {
        handed_on += w[k];
      }
    }
  }
#pragma unroll
  for (int i = 0; i < VPL; ++i) {
    if (p.h) s[i] = mcn_fma(handed_on, hv[i], s[i]);
    if (p.shared) s[i] = mcn_fma(1.f / (1.f + expf(-gate)), sv[i], s[i]);
  }
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < VPL; ++i) {
    if (p.accumulate) x[i] = mcn_fma(1.f, x[i], s[i]);
    else x[i] = s[i];
    if (p.add) x[i] = mcn_fma(1.f, mcn_load4(p.add + (size_t)n * E + at[i]), x[i]);
    if (p.vec) x[i] = mcn_fma(1.f, mcn_load4(p.vec + at[i]), x[i]);
    const bool in = (lane + i * DA_WAVE) * 4 < E;
    if (in) *(float4*)(p.y + (size_t)n * E + at[i]) = x[i];
    else x[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    sum += (x[i].x + x[i].y) + (x[i].z + x[i].w);
  }
  const float mean = p.centre ? wave_sum(sum) / (float)E : 0.f;
  float q = 0.f;
#pragma unroll
  for (int i = 0; i < VPL; ++i) {
    const bool in = (lane + i * DA_WAVE) * 4 < E;
    x[i] = make_float4(x[i].x - mean, x[i].y - mean, x[i].z - mean, x[i].w - mean);
    if (in) q += (x[i].x * x[i].x + x[i].y * x[i].y) + (x[i].z * x[i].z + x[i].w * x[i].w);
  }
  const float inv = 1.0f / sqrtf(wave_sum(q) / (float)E + p.eps);
#pragma unroll
  for (int i = 0; i < VPL; ++i) {
    if ((lane + i * DA_WAVE) * 4 >= E) continue;
    const float4 o = make_float4(x[i].x * inv * (p.offset + g[i].x) + b[i].x, x[i].y * inv * (p.offset + g[i].y) + b[i].y,
                                 x[i].z * inv * (p.offset + g[i].z) + b[i].z, x[i].w * inv * (p.offset + g[i].w) + b[i].w);
    if (sizeof(T) == 2) *(uint2*)((bf16_t*)p.h_next + (size_t)n * E + at[i]) = make_uint2(pack2_bf16(o.x, o.y), pack2_bf16(o.z, o.w));
    else *(float4*)((float*)p.h_next + (size_t)n * E + at[i]) = o;
  }
}

extern "C" int da_moe_combine_norm_takes(int width) { return width > 0 && width % 4 == 0 && width <= 4096; }

extern "C" int da_moe_combine_norm(const float* out, int ldo, const int* slot_of_pair, const float* weights, float uniform, int top,
                                   float* y, int N, int width, int accumulate, const void* h, int ldh, const float* shared, int lds,
                                   const float* gate, int ldg, const float* add, const float* vec, const void* gain, int gain_dtype,
                                   const void* bias, int bias_dtype, float offset, float eps, int centre, void* h_next, int dtype,
                                   void* stream) {
  DA_REQUIRE(N >= 0 && da_moe_combine_norm_takes(width) && top > 0 && ldo >= width && ldo % 4 == 0, "moe_combine_norm: bad sizes");
  DA_REQUIRE((!h || (ldh >= width && ldh % 4 == 0)) && (!shared || (lds >= width && lds % 4 == 0 && gate && ldg > 0)), "moe_combine_norm: row lengths");
  DA_REQUIRE(eps > 0.f && gain && h_next && h_next != h, "moe_combine_norm: eps must be > 0, and the next norm needs a gain and rows of its own");
  DA_REQUIRE((((uintptr_t)out | (uintptr_t)y | (uintptr_t)h | (uintptr_t)shared | (uintptr_t)add | (uintptr_t)vec | (uintptr_t)gain |
               (uintptr_t)bias | (uintptr_t)h_next) % 16) == 0, "moe_combine_norm: operands must be 16-byte aligned");
  if (N == 0) return 0;
  const CombineNorm p{out, ldo, slot_of_pair, weights, uniform, top, y, h, ldh, shared, lds, gate, ldg, add, vec, gain, gain_dtype,
                      bias, bias_dtype, offset, eps, centre, h_next, N, width, accumulate};
  const int wpb = N >= 512 ? 4 : 1;
  const dim3 grid(da_ceil_div(N, wpb)), block(wpb * DA_WAVE);
#define MCN_GO(V)                                                                                                         \
  do {                                                                                                                    \
    if (dtype == DA_BF16) hipLaunchKernelGGL((moe_combine_norm_kernel<bf16_t, V>), grid, block, 0, (hipStream_t)stream, p); \
    else hipLaunchKernelGGL((moe_combine_norm_kernel<float, V>), grid, block, 0, (hipStream_t)stream, p);                  \
  } while (0)
  if (width <= 256) MCN_GO(1);
  else if (width <= 512) MCN_GO(2);
  else if (width <= 1024) MCN_GO(4);
  else if (width <= 2048) MCN_GO(8);
  else MCN_GO(16);
#undef MCN_GO
  DA_CHECK_LAUNCH("moe_combine_norm");
  return 0;
}

// ---- the grouped products on the matrix cores (bfloat16) ---------------------------------------------------
// A workgroup owns a tile of 32 slots x 16 columns of one expert, and its wavefronts share out k: wavefront v takes the
// k-steps of 32 number v, v + NW, ... with MFMA 16x16x32, operands from memory into the lanes' fragments (a lane's 16 bytes
// are 8 consecutive k of one row), MM_UNROLL steps asked for at once.  With few rows an expert, as in decoding, the kernel
// streams the expert's weights once, and narrow columns mean many workgroups for that (8 experts of 512 x 768: 256).  The
// wavefronts' sums meet in LDS and are added in the order of the wavefronts.  GATED: the gate and up rows of the same
// columns are multiplied side by side and out = act(g) * u leaves in bfloat16; else one product leaves in 32-bit.  A row's
// sums run in one order whatever else is in the step.  Measured on MI355X against 64 columns a workgroup without shared k
// (8 tokens, 2 of 8 experts of 512 x 768): 10.7 -> 5.7 us, down 6.2 -> 5.3.
#define MM_ROWS 32
#define MM_COLS 16
#define MM_UNROLL 4

template <int MODE, int NW>
__global__ void __launch_bounds__(NW * DA_WAVE)
moe_mfma_kernel(const bf16_t* __restrict__ a, int lda, const int* __restrict__ row_of_slot,
                const int* __restrict__ tile_expert, const bf16_t* __restrict__ w, void* __restrict__ out, int ldo,
                int K, int F, int act, const float* __restrict__ slot_scale, float limit) {
  constexpr bool GATED = MODE == MOE_GATED, GATHER = MODE != MOE_DOWN;
  constexpr int G = GATED ? 2 : 1;
  __shared__ float sums[NW][G][8][DA_WAVE];                 // [wavefront][product][register of the tile][lane]
  const int t = threadIdx.x, lane = t % DA_WAVE, wave = t / DA_WAVE;
  const int fr = lane % 16, fk = (lane / 16) * 8;
  const int m0 = blockIdx.y * MM_ROWS, n0 = blockIdx.x * MM_COLS;
  // every load of the routing at once: the expert, the rows of a, the rows that this thread will store
  constexpr int PER = (8 + NW - 1) / NW;
  const int e = tile_expert[blockIdx.y];
  int srow[2], used[PER];
#pragma unroll
  for (int i = 0; i < 2; ++i) srow[i] = row_of_slot[m0 + i * 16 + fr];
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int x = (wave + j * NW) % 8;
    used[j] = row_of_slot[m0 + x / 4 * 16 + 4 * (lane / 16) + x % 4];
  }
  if (e < 0) return;
  // the rows of a: gathered by slot for the first product (a padding slot reads row 0 and is never stored),
  // the slot's own row for the second; an expert's slots are filled from the front
  const bool two = __builtin_amdgcn_readfirstlane(srow[1]) >= 0;      // (lane 0's: slot m0 + 16; the same for the workgroup)
  const bf16_t* ap[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = GATHER ? (srow[i] >= 0 ? srow[i] : 0) : m0 + i * 16 + fr;
    ap[i] = a + (size_t)r * lda + fk;
  }
  const int wcol = n0 + fr < F ? n0 + fr : 0;
  const bf16_t* wg = w + ((size_t)e * G * F + wcol) * K + fk;
  const bf16_t* wu = wg + (size_t)F * K;
  floatx4 acc[2][G];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int g = 0; g < G; ++g) acc[i][g] = floatx4{0.f, 0.f, 0.f, 0.f};
  const uint4 zero = make_uint4(0, 0, 0, 0);
  for (int k0 = wave * 32; k0 < K; k0 += 32 * NW * MM_UNROLL) {
    uint4 av[MM_UNROLL][2], wv[MM_UNROLL][G];
#pragma unroll
    for (int u = 0; u < MM_UNROLL; ++u) {
      const int k = k0 + u * 32 * NW;
      const int ks = (k + fk < K) ? k : -fk;                // past K: the row's first chunk, met by zeros in a
      wv[u][0] = load16(wg + ks);
      if (GATED) wv[u][G - 1] = load16(wu + ks);
      av[u][0] = load16(ap[0] + ks);
      av[u][1] = two ? load16(ap[1] + ks) : zero;
    }
#pragma unroll
    for (int u = 0; u < MM_UNROLL; ++u) {
      const bool kin = k0 + u * 32 * NW + fk < K;
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        if (i == 1 && !two) continue;
        const uint4 x = kin ? av[u][i] : zero;
#pragma unroll
        for (int g = 0; g < G; ++g)
          acc[i][g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_t, x),
                                                              __builtin_bit_cast(bf16x8_t, wv[u][g]), acc[i][g], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int g = 0; g < G; ++g)
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) sums[wave][g][i * 4 + r][lane] = acc[i][g][r];
  lds_barrier();
  // acc[i][.][r] of a lane is row 16 i + 4 (lane / 16) + r of the tile, column n0 + lane % 16
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int x = wave + j * NW;
    const int row = x / 4 * 16 + 4 * (lane / 16) + x % 4;
    if (x >= 8 || used[j] < 0 || n0 + fr >= F) continue;
    float v[G];
#pragma unroll
    for (int g = 0; g < G; ++g) {
      v[g] = sums[0][g][x][lane];
#pragma unroll
      for (int k = 1; k < NW; ++k) v[g] += sums[k][g][x][lane];
    }
    const size_t o = (size_t)(m0 + row) * ldo + n0 + fr;
    const float sc = (GATHER && slot_scale) ? slot_scale[m0 + row] : 1.0f;
    if (GATED) ((bf16_t*)out)[o] = f32_to_bf16(gated_mid<true>(sc * v[0], sc * v[G - 1], act, limit));
    else if (MODE == MOE_UP) ((bf16_t*)out)[o] = f32_to_bf16(apply_act_bf16(sc * v[0], act));
    else ((float*)out)[o] = v[0];
  }
}

// eight wavefronts where k has steps for them, else four
#define MM_LAUNCH(MODE, cols, K, ...)                                                                                        \
  do {                                                                                                                       \
    const dim3 grid_(da_ceil_div(cols, MM_COLS), T_cap);                                                                     \
    if ((K) > 128) hipLaunchKernelGGL((moe_mfma_kernel<MODE, 8>), grid_, dim3(8 * DA_WAVE), 0, (hipStream_t)stream, __VA_ARGS__); \
    else hipLaunchKernelGGL((moe_mfma_kernel<MODE, 4>), grid_, dim3(4 * DA_WAVE), 0, (hipStream_t)stream, __VA_ARGS__);      \
  } while (0)

static int moe_mfma_checks(const void* a, int lda, const void* w, int K, const char* name) {
  DA_REQUIRE(K % 8 == 0 && lda % 8 == 0 && (uintptr_t)a % 16 == 0 && (uintptr_t)w % 16 == 0,
             "%s: K and the row length of a must be multiples of 8, operands 16-byte aligned", name);
  return 0;
}

extern "C" int da_moe_tile_rows_mfma() { return MM_ROWS; }

extern "C" int da_moe_gated_mfma(const void* a, int lda, const int* row_of_slot, const int* tile_expert, const void* w,
                                 void* mid, int ldm, int T_cap, int K, int F, int act, float limit, void* stream) {
  DA_REQUIRE(T_cap >= 0 && K > 0 && F > 0 && lda >= K && ldm >= F, "moe_gated_mfma: bad sizes");
  DA_REQUIRE(act != DA_ACT_GLU_CAPPED || limit > 0.f, "moe_gated_mfma: the capped form needs a positive limit");
  DA_REQUIRE(act >= DA_ACT_NONE && act <= DA_ACT_LAST, "moe_gated_mfma: unknown activation %d", act);
  if (moe_mfma_checks(a, lda, w, K, "moe_gated_mfma")) return 1;
  if (T_cap == 0) return 0;
  MM_LAUNCH(MOE_GATED, F, K, (const bf16_t*)a, lda, row_of_slot, tile_expert, (const bf16_t*)w, mid, ldm, K, F, act, nullptr, limit);
  DA_CHECK_LAUNCH("moe_gated_mfma");
  return 0;
}

extern "C" int da_moe_up_mfma(const void* a, int lda, const int* row_of_slot, const int* tile_expert, const void* w,
                              const float* slot_scale, void* mid, int ldm, int T_cap, int K, int F, int act, void* stream) {
  DA_REQUIRE(T_cap >= 0 && K > 0 && F > 0 && lda >= K && ldm >= F, "moe_up_mfma: bad sizes");
  DA_REQUIRE(act >= DA_ACT_NONE && act <= DA_ACT_LAST, "moe_up_mfma: unknown activation %d", act);
  if (moe_mfma_checks(a, lda, w, K, "moe_up_mfma")) return 1;
  if (T_cap == 0) return 0;
  MM_LAUNCH(MOE_UP, F, K, (const bf16_t*)a, lda, row_of_slot, tile_expert, (const bf16_t*)w, mid, ldm, K, F, act, slot_scale, 0.f);
  DA_CHECK_LAUNCH("moe_up_mfma");
  return 0;
}

extern "C" int da_moe_down_mfma(const void* mid, int ldm, const int* row_of_slot, const int* tile_expert, const void* w,
                                float* out, int ldo, int T_cap, int F, int width, void* stream) {
  DA_REQUIRE(T_cap >= 0 && F > 0 && width > 0 && ldm >= F && ldo >= width, "moe_down_mfma: bad sizes");
  if (moe_mfma_checks(mid, ldm, w, F, "moe_down_mfma")) return 1;
  if (T_cap == 0) return 0;
  MM_LAUNCH(MOE_DOWN, width, F, (const bf16_t*)mid, ldm, row_of_slot, tile_expert, (const bf16_t*)w, out, ldo, F, width, 0,
            nullptr, 0.f);
  DA_CHECK_LAUNCH("moe_down_mfma");
  return 0;
}

// rows of a in the order of the slots (zeros for slots that hold no pair): the operand of the grouped block-tile
// product, 16 bytes a thread
__global__ void moe_gather_kernel(const bf16_t* __restrict__ a, int lda, const int* __restrict__ row_of_slot,
                                  bf16_t* __restrict__ out, int rows, int width8, const float* __restrict__ slot_scale) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= (long)rows * width8) return;
  const int slot = (int)(i / width8), c = (int)(i % width8) * 8;
  const int r = row_of_slot[slot];
  uint4 v = make_uint4(0, 0, 0, 0);
  if (r >= 0) v = *(const uint4*)(a + (size_t)r * lda + c);
  if (slot_scale && r >= 0) {                     // the row times its pair's weight, rounded once
    const float sc = slot_scale[slot];
    uint32_t* w2 = (uint32_t*)&v;
#pragma unroll
    for (int e = 0; e < 4; ++e)
      w2[e] = pack2_bf16(sc * bf16_to_f32((bf16_t)(w2[e] & 0xffffu)), sc * bf16_to_f32((bf16_t)(w2[e] >> 16)));
  }
  *(uint4*)(out + (size_t)slot * width8 * 8 + c) = v;
}

extern "C" int da_moe_gather(const void* a, int lda, const int* row_of_slot, void* out, int rows, int width, void* stream,
                             const float* slot_scale) {
  DA_REQUIRE(rows >= 0 && width > 0 && width % 8 == 0 && lda % 8 == 0 && lda >= width, "moe_gather: the width must be a multiple of 8");
  DA_REQUIRE((uintptr_t)a % 16 == 0 && (uintptr_t)out % 16 == 0, "moe_gather: operands must be 16-byte aligned");
  if (rows == 0) return 0;
  const long n = (long)rows * (width / 8);
  hipLaunchKernelGGL(moe_gather_kernel, dim3(da_ceil_div(n, 256)), dim3(256), 0, (hipStream_t)stream, (const bf16_t*)a, lda,
                     row_of_slot, (bf16_t*)out, rows, width / 8, slot_scale);
  DA_CHECK_LAUNCH("moe_gather");
  return 0;
}
