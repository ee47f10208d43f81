// Gated linear attention: linear attention with a decay per head and key channel that the input sets.
//
// Per head h a matrix S [D rows (key channels)][Dv columns (value channels)], 32-bit, token by token:
//     S <- diag(a) S + k v^T        a[d] = logistic(z[d])^(1 / tau),  z = raw[d] + bias[d]
//     o  = S^T (q_scale q)          (after the write)
//
// The walk (`da_gla_walk`; both dtypes, any portion, D up to 256): the columns of S do not meet, so a column is shared
// out over 16 neighbouring lanes, lane j holding the RPL consecutive rows from j * RPL on in registers; the sum over
// rows is taken inside the lane and then over the 16 lanes by DPP additions.  A workgroup holds 16 columns of a head and
// walks its sequence's portion in order; the grid is (column blocks x heads x sequences).  Tokens come through LDS in
// blocks, the decays worked out once a (token, row) as they are parked; every thread asks for its share of the next
// block before it walks the block at hand.  A token's result is the same bits however the sequence was cut into steps
// and whatever else the step holds.
//
// A request's state row holds S as [H][Dv][D] (a column's rows side by side) at its start; a sequence without a slot (a
// padding row of a fixed-shape step) starts from zeros and keeps nothing.
#include "common.h"

#define GLA_LPC 16            // lanes that share a column in the walk
#define GLA_CPB 16            // columns of a walking workgroup
#define GLA_MAX_D 256
#define GLA_LOG2E 1.4426950408889634f

// log2 of the decay: log2(logistic(z)) / tau
template <bool FAST>
__device__ __forceinline__ float gla_log2_decay(float z, float inv_tau) {
  if (FAST) {
    const float y = z * GLA_LOG2E;
    return (fminf(y, 0.f) - __builtin_amdgcn_logf(1.0f + __builtin_amdgcn_exp2f(-fabsf(y)))) * inv_tau;
  }
  return (fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * (inv_tau * GLA_LOG2E);
}
template <bool FAST>
__device__ __forceinline__ float gla_decay(float z, float inv_tau) {
  if (FAST) return __builtin_amdgcn_exp2f(gla_log2_decay<true>(z, inv_tau));
  return expf((fminf(z, 0.f) - log1pf(expf(-fabsf(z)))) * inv_tau);
}

struct GlaArgs {
  const void* qkv; int ld;            // [N, ...]: q at q_off, k at k_off (H * D each), v at v_off (H * Dv)
  int q_off, k_off, v_off;
  const float* raw; int raw_ld;       // [N, H * D]: the decays' arguments before their bias
  const float* bias;                  // [H * D]
  float* state; long state_ld;        // [slots, >= H * Dv * D]
  const int* state_slots;             // [S]
  const int* q_start;                 // [S + 1]
  float* o; int o_ld;                 // [N, H * Dv]
  int H, D, Dv, write;
  float q_scale, inv_tau;
};

template <typename T, int RPL, bool FAST>
__global__ void __launch_bounds__(GLA_CPB * GLA_LPC)
gla_walk_kernel(GlaArgs A) {
  constexpr int DP = RPL * GLA_LPC;                 // D rounded up to what the lanes hold
  constexpr int TB = RPL <= 4 ? 32 : (RPL <= 8 ? 16 : 8);        // tokens of a block
  constexpr int PER = TB * RPL / GLA_LPC;           // entries of q (of k, of the decays) of a block that a thread brings
  constexpr int PERV = (TB + 15) / 16;              // ... and of v
  __shared__ __attribute__((aligned(16))) float qs[TB][DP], ks[TB][DP], as[TB][DP], vs[TB][GLA_CPB];
  const int t = threadIdx.x, j = t % GLA_LPC, c = t / GLA_LPC;
  const int h = blockIdx.y, s = blockIdx.z;
  const int col = blockIdx.x * GLA_CPB + c;
  const bool col_ok = col < A.Dv;
  const int row0 = A.q_start[s], n_tok = A.q_start[s + 1] - row0;
  if (n_tok <= 0) return;
  const int slot = A.state_slots[s];
  const T* base = (const T*)A.qkv;
  float* srow = (slot >= 0 && col_ok) ? A.state + (size_t)slot * A.state_ld + ((size_t)h * A.Dv + col) * A.D : nullptr;
  float S[RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const int r = j * RPL + i;
    S[i] = (srow && r < A.D) ? srow[r] : 0.f;
  }
  // this thread's share of a block: entries t + 256 i of [token][DP] for q, k and the decays, of [token][16] for v;
  // loads are unconditional, from places that exist, and looked at when they are parked
  T rq[PER], rk[PER], rv[PERV];
  float ra[PER];
  auto fetch = [&](int t0) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int idx = t + 256 * i, tok = idx / DP, r = idx % DP;
      const int n = row0 + (t0 + tok < n_tok ? t0 + tok : 0), d = h * A.D + (r < A.D ? r : 0);
      rq[i] = base[(size_t)n * A.ld + A.q_off + d];
      rk[i] = base[(size_t)n * A.ld + A.k_off + d];
      ra[i] = A.raw[(size_t)n * A.raw_ld + d] + A.bias[d];
    }
#pragma unroll
    for (int i = 0; i < PERV; ++i) {
      const int idx = t + 256 * i, tok = idx / GLA_CPB, cc = blockIdx.x * GLA_CPB + idx % GLA_CPB;
      rv[i] = base[(size_t)(row0 + (t0 + tok < n_tok ? t0 + tok : 0)) * A.ld + A.v_off + (size_t)h * A.Dv + (cc < A.Dv ? cc : 0)];
    }
  };
  auto park = [&](int nt) {                         // (tokens past the block's last are never read)
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int idx = t + 256 * i, tok = idx / DP, r = idx % DP;
      const bool e = r < A.D;
      if (tok < nt) {
        qs[tok][r] = e ? to_f32(rq[i]) * A.q_scale : 0.f;
        ks[tok][r] = e ? to_f32(rk[i]) : 0.f;
        as[tok][r] = e ? gla_decay<FAST>(ra[i], A.inv_tau) : 1.f;
      }
    }
#pragma unroll
    for (int i = 0; i < PERV; ++i) {
      const int idx = t + 256 * i;
      if (idx / GLA_CPB < nt) vs[idx / GLA_CPB][idx % GLA_CPB] = to_f32(rv[i]);
    }
  };

  fetch(0);
  for (int t0 = 0; t0 < n_tok; t0 += TB) {
    const int nt = n_tok - t0 < TB ? n_tok - t0 : TB;
    __syncthreads();                                // the block before has been walked by everyone
    park(nt);
    __syncthreads();
    if (t0 + TB < n_tok) fetch(t0 + TB);
    for (int k = 0; k < nt; ++k) {
      const float vv = vs[k][c];
      float acc = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        const int r = j * RPL + i;
        S[i] = fmaf(as[k][r], S[i], ks[k][r] * vv);
        acc = fmaf(S[i], qs[k][r], acc);
      }
      acc = group_sum<GLA_LPC>(acc);
      if (j == 0 && col_ok) A.o[(size_t)(row0 + t0 + k) * A.o_ld + (size_t)h * A.Dv + col] = acc;
    }
  }
  if (srow && A.write) {
#pragma unroll
    for (int i = 0; i < RPL; ++i) {
      const int r = j * RPL + i;
      if (r < A.D) srow[r] = S[i];
    }
  }
}

template <typename T, bool FAST>
static int gla_walk_go(const GlaArgs& A, int S, void* stream) {
  const dim3 grid((unsigned)da_ceil_div(A.Dv, GLA_CPB), (unsigned)A.H, (unsigned)S), block(GLA_CPB * GLA_LPC);
  hipStream_t st = (hipStream_t)stream;
  const int rpl = da_ceil_div(A.D, GLA_LPC);
  if (rpl <= 1) hipLaunchKernelGGL((gla_walk_kernel<T, 1, FAST>), grid, block, 0, st, A);
  else if (rpl <= 2) hipLaunchKernelGGL((gla_walk_kernel<T, 2, FAST>), grid, block, 0, st, A);
  else if (rpl <= 4) hipLaunchKernelGGL((gla_walk_kernel<T, 4, FAST>), grid, block, 0, st, A);
  else if (rpl <= 8) hipLaunchKernelGGL((gla_walk_kernel<T, 8, FAST>), grid, block, 0, st, A);
  else hipLaunchKernelGGL((gla_walk_kernel<T, 16, FAST>), grid, block, 0, st, A);
  DA_CHECK_LAUNCH("gla_walk");
  return 0;
}

// Sequences 0 .. S - 1 of the step; rows of sequence s are q_start[s] .. q_start[s + 1] - 1.  The state row of
// state_slots[s] is read at the portion's start and, with `write`, written at its end.
extern "C" int da_gla_walk(const void* qkv, int dtype, int ld, int q_off, int k_off, int v_off, const float* raw, int raw_ld,
                           const float* bias, float tau, float q_scale, float* state, long state_ld, const int* state_slots,
                           const int* q_start, float* o, int o_ld, int S, int H, int D, int Dv, int write, void* stream) {
  DA_REQUIRE(S >= 0 && H > 0 && D > 0 && Dv > 0, "gla_walk: bad sizes");
  DA_REQUIRE(D <= GLA_MAX_D, "gla_walk: a key size of %d, %d are taken", D, GLA_MAX_D);
  DA_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && ld >= q_off + H * D && ld >= k_off + H * D && ld >= v_off + H * Dv,
             "gla_walk: q, k and v leave the row");
  DA_REQUIRE(raw_ld >= H * D && o_ld >= H * Dv && state_ld >= (long)H * Dv * D, "gla_walk: row lengths too small");
  DA_REQUIRE(tau > 0.f, "gla_walk: tau must be positive, found %g", (double)tau);
  DA_REQUIRE(H <= 65535 && S <= 65535, "gla_walk: too many heads or sequences for one launch");
  if (S == 0) return 0;
  GlaArgs A;
  A.qkv = qkv; A.ld = ld; A.q_off = q_off; A.k_off = k_off; A.v_off = v_off; A.raw = raw; A.raw_ld = raw_ld; A.bias = bias;
  A.state = state; A.state_ld = state_ld; A.state_slots = state_slots; A.q_start = q_start; A.o = o; A.o_ld = o_ld;
  A.H = H; A.D = D; A.Dv = Dv; A.write = write; A.q_scale = q_scale; A.inv_tau = 1.0f / tau;
  if (dtype == DA_BF16) return gla_walk_go<bf16_t, true>(A, S, stream);
  return gla_walk_go<float, false>(A, S, stream);
}
