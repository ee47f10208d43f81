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
// In bfloat16 serving, for key and value sizes up to 128 (the key size a multiple of 4), two other forms, which also
// divide each head's read-out by its root mean square and multiply it with the gain and the gate, so that what leaves
// them is the output projection's input:
//   `da_gla_decode`  sequences that bring one token: a workgroup a (sequence, head), every state entry read and written
//                    once in 16-byte pieces.
//   `da_gla_chunked` portions, in chunks of 64 tokens that run side by side (three launches).  With G_b the product of
//                    the decays of a block of 16 tokens and everything row by row:
//     states  chunk c from a zero state: Q_c = sum_s (k_s times the decays behind s) v_s^T, block by block,
//             acc <- G_b acc + K_b^T V_b on the 32-bit matrix cores; and the chunk's whole decay
//     carry   start_0 = the request's state, start_(c+1) = decay_c start_c + Q_c; the last one is kept
//     output  a wavefront a block of 16 rows: o = (A masked) V inside the block, then the blocks before it in the chunk,
//             then the chunk's start state; queries carry the decays back to the block at hand, keys the decays on to
//             their block's end, so that every factor is a decay (at most 1).  Inside a block the queries are divided
//             by the block's whole decay instead; where that is too small to divide by (below 2^-100), the block's
//             scores are summed pair by pair with the decay between the two tokens.
//   All of it is 32-bit: decays and their logarithms, the products' operands and sums, states.  A row's result depends
//   on where its chunk starts in the portion by 32-bit rounding only.
// Both take the decays' arguments as rows of their own, or work them out from the low rank (`up`, up to 32 numbers).
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

// ---------------------------------------------------------------------------------------- bfloat16 serving
#define GLA_CHUNK 64
#define GLA_BLK 16
#define GLA_NBLK (GLA_CHUNK / GLA_BLK)
#define GLA_LOW_MAX 32        // numbers of the decay's low rank that the kernels multiply up themselves
#define GLA_SERVE_D 128
#define GLA_THIN -100.f       // log2 of a block's decay below which its scores are summed pair by pair

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float gla_floatx4;

struct GlaServeArgs {
  const bf16_t* proj; int ld;         // [N, ...]: q, k, v, gate and the low rank's numbers at these columns
  int q_off, k_off, v_off, g_off, low_off;
  const bf16_t* up; int rank;         // [H * D, rank], or null: the arguments are in raw
  const float* raw; int raw_ld;       // [N, H * D]
  const float* bias;                  // [H * D]
  const void* gain; int gain_dtype;   // [Dv]
  float* state; long state_ld;
  const int* state_slots; const int* q_start;
  bf16_t* y; int y_ld;                // [N, H * Dv]
  int H, D, Dv, write, seq0, n_seqs;
  float q_scale, inv_tau, eps;
  int whole_qk, whole_v, whole_low;   // four entries of q and k, of v, of the low rank's numbers lie 8-byte aligned
  int n_chunks;                       // chunks of the longest portion
  float* ends;                        // [n_seqs, n_chunks, H, Dv, D]: chunks' end states, then their start states
  float* chunk_decay;                 // [n_seqs, n_chunks, H, D]
};

// ---- one token a sequence: a workgroup a (sequence, head), a column over 16 lanes, 16 columns at a time
template <int RPL>
__global__ void __launch_bounds__(256)
gla_decode_kernel(GlaServeArgs A) {
  constexpr int NP = GLA_SERVE_D / 16;              // passes over the columns at most
  constexpr int AHEAD = RPL <= 4 ? 4 : 2;           // passes whose state is asked for at once
  constexpr int Q4 = RPL / 4;
  __shared__ __attribute__((aligned(16))) float qs[GLA_SERVE_D], ks[GLA_SERVE_D], as[GLA_SERVE_D];
  __shared__ float vs[GLA_SERVE_D], os[GLA_SERVE_D], part[4];
  const int t = threadIdx.x, j = t % 16, c = t / 16;
  const int h = blockIdx.x % A.H, s = A.seq0 + blockIdx.x / A.H;
  const int n = A.q_start[s];
  if (A.q_start[s + 1] <= n) return;                // (the whole workgroup)
  const int slot = A.state_slots[s];
  const bf16_t* row = A.proj + (size_t)n * A.ld;
  const int hd = h * A.D;
  const int np = (A.Dv + 15) / 16;
  float* st = A.state + (size_t)(slot >= 0 ? slot : 0) * A.state_ld + (size_t)h * A.Dv * A.D;
  float4 S[NP][Q4];
  auto fetch = [&](int p0) {
#pragma unroll
    for (int p = p0; p < p0 + AHEAD; ++p) {
      if (p >= NP) continue;
      const int col = p * 16 + c;
#pragma unroll
      for (int i = 0; i < Q4; ++i) {
        const int r = j * RPL + 4 * i;
        const bool ok = slot >= 0 && col < A.Dv && r < A.D;
        float4 v = *(const float4*)(st + (size_t)(col < A.Dv ? col : 0) * A.D + (r < A.D ? r : 0));
        if (!ok) v = make_float4(0.f, 0.f, 0.f, 0.f);
        S[p][i] = v;
      }
    }
  };
  fetch(0);
  if (t < A.D) {
    qs[t] = bf16_to_f32(row[A.q_off + hd + t]) * A.q_scale;
    ks[t] = bf16_to_f32(row[A.k_off + hd + t]);
    float z = A.bias[hd + t];
    if (A.up) {
      for (int r = 0; r < A.rank; r += 4) {
        const uint2 w = *(const uint2*)(A.up + (size_t)(hd + t) * A.rank + r);
        const bf16_t* lo = row + A.low_off + r;
        z = fmaf(bf16_to_f32((bf16_t)(w.x & 0xffffu)), bf16_to_f32(lo[0]), z);
        z = fmaf(bf16_to_f32((bf16_t)(w.x >> 16)), bf16_to_f32(lo[1]), z);
        z = fmaf(bf16_to_f32((bf16_t)(w.y & 0xffffu)), bf16_to_f32(lo[2]), z);
        z = fmaf(bf16_to_f32((bf16_t)(w.y >> 16)), bf16_to_f32(lo[3]), z);
      }
    } else {
      z += A.raw[(size_t)n * A.raw_ld + hd + t];
    }
    as[t] = gla_decay<true>(z, A.inv_tau);
  } else if (t < GLA_SERVE_D) {
    qs[t] = 0.f; ks[t] = 0.f; as[t] = 1.f;
  }
  float gate = 0.f, gain = 0.f;
  if (t < A.Dv) {
    vs[t] = bf16_to_f32(row[A.v_off + h * A.Dv + t]);
    gate = bf16_to_f32(row[A.g_off + h * A.Dv + t]);
    gain = load_param(A.gain, A.gain_dtype, t);
  } else if (t < GLA_SERVE_D) {
    vs[t] = 0.f;
  }
  lds_barrier();
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    if (p < np) {
      if (p % AHEAD == 0 && p) fetch(p);
      const int col = p * 16 + c;
      const float v = vs[col];
      float acc = 0.f;
#pragma unroll
      for (int i = 0; i < Q4; ++i) {
        const int r = j * RPL + 4 * i;
        const float4 a = *(const float4*)(as + r), k = *(const float4*)(ks + r), q = *(const float4*)(qs + r);
        float4 x = S[p][i];
        x.x = fmaf(a.x, x.x, k.x * v);
        x.y = fmaf(a.y, x.y, k.y * v);
        x.z = fmaf(a.z, x.z, k.z * v);
        x.w = fmaf(a.w, x.w, k.w * v);
        acc = fmaf(x.x, q.x, acc);
        acc = fmaf(x.y, q.y, acc);
        acc = fmaf(x.z, q.z, acc);
        acc = fmaf(x.w, q.w, acc);
        if (A.write && slot >= 0 && col < A.Dv && r < A.D) *(float4*)(st + (size_t)col * A.D + r) = x;
      }
      acc = group_sum<16>(acc);
      if (j == 0) os[col] = acc;
    }
  }
  lds_barrier();
  // the read-out's norm, gain and gate
  const float o = t < A.Dv ? os[t] : 0.f;
  const float ss = wave_sum(o * o);
  if (t % DA_WAVE == 0) part[t / DA_WAVE] = ss;
  lds_barrier();
  if (t < A.Dv) {
    const float inv = 1.0f / sqrtf((part[0] + part[1] + part[2] + part[3]) / (float)A.Dv + A.eps);
    const float g = gate * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-GLA_LOG2E * gate));
    A.y[(size_t)n * A.y_ld + h * A.Dv + t] = f32_to_bf16(o * inv * gain * g);
  }
}

// ---- portions in chunks
// What both passes over the tokens start from, for the chunk of n tokens whose first row is n0: keys times the decays
// up to their block's end, values, the blocks' whole decays, and (for the output pass) queries times the decays since
// their block's start, and the running logarithms.  A thread takes a (block, row of the state).
template <int DT, int VT, bool OUT>
struct GlaLds {
  static constexpr int DP = DT * 16, DS = DP + 4;   // an odd number of 16-byte pieces a row: 16 rows fall on different banks
  static constexpr int VP = VT * 16, VS = VP + 4;
  float kh[GLA_CHUNK * DS];
  float qh[OUT ? GLA_CHUNK * DS : 4];
  float la[OUT ? GLA_CHUNK * DS : GLA_CHUNK * GLA_LOW_MAX];   // first the low rank's numbers, then the logarithms
  float G[GLA_NBLK * DP];
  bf16_t v[GLA_CHUNK * VS];
  int thin[GLA_NBLK];
};

// Four neighbouring entries of a row of proj; `whole`: one 8-byte load (the same for the whole launch).
__device__ __forceinline__ uint2 gla_load4(const bf16_t* row, int at, int count, bool whole) {
  if (whole) return *(const uint2*)(row + (at < count ? at : 0));
  uint32_t e[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) e[i] = row[at + i < count ? at + i : 0];
  return make_uint2(e[0] | (e[1] << 16), e[2] | (e[3] << 16));
}
// ... with zeros for what lies behind the row's last entry, or everywhere
__device__ __forceinline__ uint2 gla_keep4(uint2 x, int at, int count, bool any) {
  if (!any || at >= count) return make_uint2(0, 0);
  if (at + 1 >= count) x.x &= 0xffffu;
  if (at + 2 >= count) x.y = 0;
  else if (at + 3 >= count) x.y &= 0xffffu;
  return x;
}
__device__ __forceinline__ float4 gla_widen4(uint2 x) {
  return make_float4(__uint_as_float(x.x << 16), __uint_as_float(x.x & 0xffff0000u), __uint_as_float(x.y << 16),
                     __uint_as_float(x.y & 0xffff0000u));
}

template <int DT, int VT, bool OUT>
__device__ __forceinline__ void gla_prepare(const GlaServeArgs& A, GlaLds<DT, VT, OUT>& L, int h, int n0, int n) {
  constexpr int DP = DT * 16, DS = DP + 4, VP = VT * 16, VS = VP + 4;
  constexpr int ITEMS = GLA_NBLK * DP, PER = ITEMS > 256 ? ITEMS / 256 : 1;
  constexpr int UP4 = GLA_LOW_MAX / 4, LOWN = GLA_CHUNK * UP4 / 256;
  static_assert(GLA_CHUNK * DS >= GLA_CHUNK * GLA_LOW_MAX, "the low rank's numbers lie where the logarithms go");
  const int t = threadIdx.x;
  // Every load first, from places that exist: keys, queries, values and the low rank's numbers in pieces of four
  // entries, then this thread's rows of the low rank's second matrix and their bias.
  uint2 rk[DT], rq[OUT ? DT : 1], rv[VT], rl[LOWN], up[PER][UP4];
  float bias[PER], zr[PER][GLA_BLK];
#pragma unroll
  for (int u = 0; u < DT; ++u) {
    const int idx = t + 256 * u, tok = idx / (DP / 4), d = idx % (DP / 4) * 4;
    const bf16_t* row = A.proj + (size_t)(n0 + (tok < n ? tok : 0)) * A.ld + h * A.D;
    rk[u] = gla_load4(row + A.k_off, d, A.D, A.whole_qk);
    if (OUT) rq[u] = gla_load4(row + A.q_off, d, A.D, A.whole_qk);
  }
#pragma unroll
  for (int u = 0; u < VT; ++u) {
    const int idx = t + 256 * u, tok = idx / (VP / 4), d = idx % (VP / 4) * 4;
    rv[u] = gla_load4(A.proj + (size_t)(n0 + (tok < n ? tok : 0)) * A.ld + A.v_off + h * A.Dv, d, A.Dv, A.whole_v);
  }
  if (A.up) {
#pragma unroll
    for (int u = 0; u < LOWN; ++u) {
      const int idx = t + 256 * u, tok = idx / UP4, r = idx % UP4 * 4;
      rl[u] = gla_load4(A.proj + (size_t)(n0 + (tok < n ? tok : 0)) * A.ld + A.low_off, r, A.rank, A.whole_low);
    }
  }
#pragma unroll
  for (int u = 0; u < PER; ++u) {
    const int it = t + 256 * u, b = it / DP, d = it % DP, dc = h * A.D + (d < A.D ? d : 0);
    bias[u] = A.bias[dc];
    if (A.up) {
#pragma unroll
      for (int r = 0; r < UP4; ++r)
        if (4 * r < A.rank) up[u][r] = *(const uint2*)(A.up + (size_t)dc * A.rank + 4 * r);
    } else {
#pragma unroll
      for (int i = 0; i < GLA_BLK; ++i) {
        const int tok = b * GLA_BLK + i;
        zr[u][i] = A.raw[(size_t)(n0 + (tok < n ? tok : 0)) * A.raw_ld + dc];
      }
    }
  }
  if (t < GLA_NBLK) L.thin[t] = 0;
  // keys and queries as they are go where the scaled keys will be, the low rank's numbers where the logarithms will be
  bf16_t* raw_k = (bf16_t*)L.kh;
  bf16_t* raw_q = raw_k + GLA_CHUNK * DS;
#pragma unroll
  for (int u = 0; u < DT; ++u) {
    const int idx = t + 256 * u, tok = idx / (DP / 4), d = idx % (DP / 4) * 4;
    *(uint2*)(raw_k + tok * DS + d) = gla_keep4(rk[u], d, A.D, tok < n);
    if (OUT) *(uint2*)(raw_q + tok * DS + d) = gla_keep4(rq[u], d, A.D, tok < n);
  }
#pragma unroll
  for (int u = 0; u < VT; ++u) {
    const int idx = t + 256 * u, tok = idx / (VP / 4), d = idx % (VP / 4) * 4;
    *(uint2*)(L.v + tok * VS + d) = gla_keep4(rv[u], d, A.Dv, tok < n);
  }
  if (A.up) {
#pragma unroll
    for (int u = 0; u < LOWN; ++u) {
      const int idx = t + 256 * u, tok = idx / UP4, r = idx % UP4 * 4;
      if (r < A.rank) *(float4*)(L.la + tok * GLA_LOW_MAX + r) = gla_widen4(rl[u]);
    }
  }
  lds_barrier();
  bf16_t k[PER][GLA_BLK], q[PER][OUT ? GLA_BLK : 1];
  float z[PER][GLA_BLK];
#pragma unroll
  for (int u = 0; u < PER; ++u) {
    const int it = t + 256 * u, b = it / DP, d = it % DP;
    if (it < ITEMS) {
#pragma unroll
      for (int i = 0; i < GLA_BLK; ++i) {
        k[u][i] = raw_k[(b * GLA_BLK + i) * DS + d];
        if (OUT) q[u][i] = raw_q[(b * GLA_BLK + i) * DS + d];
        z[u][i] = A.up ? 0.f : zr[u][i];
      }
      if (A.up) {
#pragma unroll
        for (int r = 0; r < UP4; ++r) {
          if (4 * r < A.rank) {
            const float4 w = gla_widen4(up[u][r]);
#pragma unroll
            for (int i = 0; i < GLA_BLK; ++i) {
              const float4 a = *(const float4*)(L.la + (b * GLA_BLK + i) * GLA_LOW_MAX + 4 * r);
              z[u][i] = fmaf(w.x, a.x, fmaf(w.y, a.y, fmaf(w.z, a.z, fmaf(w.w, a.w, z[u][i]))));
            }
          }
        }
      }
      float run = 0.f;
#pragma unroll
      for (int i = 0; i < GLA_BLK; ++i) {
        const float dec = gla_log2_decay<true>(z[u][i] + bias[u], A.inv_tau);
        run += b * GLA_BLK + i < n && d < A.D ? dec : 0.f;
        z[u][i] = run;                              // the running logarithm since the block's start
      }
    }
  }
  lds_barrier();                                    // everything parked has been read
#pragma unroll
  for (int u = 0; u < PER; ++u) {
    const int it = t + 256 * u, b = it / DP, d = it % DP;
    if (it < ITEMS) {
      const float end = z[u][GLA_BLK - 1];
      L.G[b * DP + d] = __builtin_amdgcn_exp2f(end);
      if (OUT && end < GLA_THIN) L.thin[b] = 1;
#pragma unroll
      for (int i = 0; i < GLA_BLK; ++i) {           // (keys and queries of what does not exist are zeros)
        const int tok = b * GLA_BLK + i;
        L.kh[tok * DS + d] = bf16_to_f32(k[u][i]) * __builtin_amdgcn_exp2f(end - z[u][i]);
        if (OUT) {
          L.qh[tok * DS + d] = bf16_to_f32(q[u][i]) * (A.q_scale * __builtin_amdgcn_exp2f(z[u][i]));
          L.la[tok * DS + d] = z[u][i];
        }
      }
    }
  }
  lds_barrier();
}

template <int DT, int VT>
__global__ void __launch_bounds__(256)
gla_states_kernel(GlaServeArgs A) {
  constexpr int DP = DT * 16, DS = DP + 4, VS = VT * 16 + 4, TILES = DT * VT / 4;
  __shared__ __attribute__((aligned(16))) GlaLds<DT, VT, false> L;
  const int h = blockIdx.x, kc = blockIdx.y, si = blockIdx.z, s = A.seq0 + si;
  const int n0 = A.q_start[s] + kc * GLA_CHUNK, left = A.q_start[s + 1] - n0;
  if (left <= 0) return;
  const int n = left < GLA_CHUNK ? left : GLA_CHUNK;
  gla_prepare<DT, VT, false>(A, L, h, n0, n);
  const int t = threadIdx.x, lane = t % DA_WAVE, w = t / DA_WAVE, lo = lane % 16, hi = lane / 16;
  gla_floatx4 acc[TILES];
#pragma unroll
  for (int i = 0; i < TILES; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[i][r] = 0.f;
  const int nb = (n + GLA_BLK - 1) / GLA_BLK;
  for (int b = 0; b < nb; ++b) {
#pragma unroll
    for (int i = 0; i < TILES; ++i) {
      const int vt = (w + 4 * i) % VT, dt = (w + 4 * i) / VT;
      const float4 g = *(const float4*)(L.G + b * DP + dt * 16 + 4 * hi);
      acc[i][0] *= g.x; acc[i][1] *= g.y; acc[i][2] *= g.z; acc[i][3] *= g.w;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tok = b * GLA_BLK + 4 * hi + r;
        acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(L.kh[tok * DS + dt * 16 + lo], bf16_to_f32(L.v[tok * VS + vt * 16 + lo]),
                                                      acc[i], 0, 0, 0);
      }
    }
  }
  float* ends = A.ends + ((size_t)(si * A.n_chunks + kc) * A.H + h) * A.Dv * A.D;
#pragma unroll
  for (int i = 0; i < TILES; ++i) {
    const int v = ((w + 4 * i) % VT) * 16 + lo, d = ((w + 4 * i) / VT) * 16 + 4 * hi;
    if (v < A.Dv && d < A.D) *(float4*)(ends + (size_t)v * A.D + d) = make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]);
  }
  for (int d = t; d < A.D; d += 256) {
    float all = 1.f;
    for (int b = 0; b < nb; ++b) all *= L.G[b * DP + d];
    A.chunk_decay[((size_t)(si * A.n_chunks + kc) * A.H + h) * A.D + d] = all;
  }
}

// One thread an entry of a head's state: the chunks' end states (from zero) become their true start states, and the
// request's row the state at the portion's end.
__global__ void __launch_bounds__(256)
gla_carry_kernel(GlaServeArgs A) {
  const long per = (long)A.H * A.Dv * A.D;
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= per * A.n_seqs) return;
  const int si = (int)(i / per), s = A.seq0 + si;
  const long e = i % per;
  const int n_tok = A.q_start[s + 1] - A.q_start[s];
  if (n_tok <= 0) return;
  const int nk = (n_tok + GLA_CHUNK - 1) / GLA_CHUNK;
  const int h = (int)(e / ((long)A.Dv * A.D)), d = (int)(e % A.D);
  float* ends = A.ends + (size_t)si * A.n_chunks * per + e;
  const float* dec = A.chunk_decay + ((size_t)si * A.n_chunks * A.H + h) * A.D + d;
  const int slot = A.state_slots[s];
  float* keep = A.state + (size_t)(slot >= 0 ? slot : 0) * A.state_ld + e;
  float cur = *keep;
  if (slot < 0) cur = 0.f;
  for (int k0 = 0; k0 < nk; k0 += 8) {              // eight chunks' numbers asked for at once
    float q[8], g[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int k = k0 + u < nk ? k0 + u : 0;
      q[u] = ends[(size_t)k * per];
      g[u] = dec[(size_t)k * A.H * A.D];
    }
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      if (k0 + u < nk) {
        ends[(size_t)(k0 + u) * per] = cur;
        cur = fmaf(g[u], cur, q[u]);
      }
    }
  }
  if (A.write && slot >= 0) *keep = cur;
}

template <int DT, int VT>
__global__ void __launch_bounds__(256)
gla_output_kernel(GlaServeArgs A) {
  constexpr int DP = DT * 16, DS = DP + 4, VS = VT * 16 + 4;
  constexpr bool EARLY = DT * VT <= 16;             // the start state fits into registers: asked for before anything else
  __shared__ __attribute__((aligned(16))) GlaLds<DT, VT, true> L;
  const int h = blockIdx.x, kc = blockIdx.y, si = blockIdx.z, s = A.seq0 + si;
  const int n0 = A.q_start[s] + kc * GLA_CHUNK, left = A.q_start[s + 1] - n0;
  if (left <= 0) return;
  const int n = left < GLA_CHUNK ? left : GLA_CHUNK;
  const int t = threadIdx.x, lane = t % DA_WAVE, w = t / DA_WAVE, lo = lane % 16, hi = lane / 16;
  const float* start = A.ends + ((size_t)(si * A.n_chunks + kc) * A.H + h) * A.Dv * A.D;
  auto start_piece = [&](int vt, int dt) -> float4 {
    const int v = vt * 16 + lo, d = dt * 16 + 4 * hi;
    float4 x = *(const float4*)(start + (size_t)(v < A.Dv ? v : 0) * A.D + (d < A.D ? d : 0));
    if (v >= A.Dv || d >= A.D) x = make_float4(0.f, 0.f, 0.f, 0.f);
    return x;
  };
  float4 s0[EARLY ? VT : 1][DT];
  if (EARLY) {
#pragma unroll
    for (int vt = 0; vt < VT; ++vt)
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) s0[vt][dt] = start_piece(vt, dt);
  }
  // the gates and gains of this lane's part of rows 4 hi + r
  bf16_t gate[VT][4];
  float gain[VT];
#pragma unroll
  for (int vt = 0; vt < VT; ++vt) {
    const int vc = vt * 16 + lo < A.Dv ? vt * 16 + lo : 0;
    gain[vt] = load_param(A.gain, A.gain_dtype, vc);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int tok = w * GLA_BLK + 4 * hi + r;
      gate[vt][r] = A.proj[(size_t)(n0 + (tok < n ? tok : 0)) * A.ld + A.g_off + h * A.Dv + vc];
    }
  }
  gla_prepare<DT, VT, true>(A, L, h, n0, n);
  if (w * GLA_BLK >= n) return;
  // this wavefront's rows: block w of the chunk; row lo of it as a matrix operand
  float4 qf[DT];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) qf[dt] = *(const float4*)(L.qh + (w * GLA_BLK + lo) * DS + dt * 16 + 4 * hi);
  gla_floatx4 o[VT];
#pragma unroll
  for (int vt = 0; vt < VT; ++vt)
#pragma unroll
    for (int r = 0; r < 4; ++r) o[vt][r] = 0.f;
  // scores of the block's rows (columns) with the keys of block b (rows: 4 hi + r)
  auto scores = [&](int b, const float4* qq) -> gla_floatx4 {
    gla_floatx4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const float4 k = *(const float4*)(L.kh + (b * GLA_BLK + lo) * DS + dt * 16 + 4 * hi);
      sc = __builtin_amdgcn_mfma_f32_16x16x4f32(k.x, qq[dt].x, sc, 0, 0, 0);
      sc = __builtin_amdgcn_mfma_f32_16x16x4f32(k.y, qq[dt].y, sc, 0, 0, 0);
      sc = __builtin_amdgcn_mfma_f32_16x16x4f32(k.z, qq[dt].z, sc, 0, 0, 0);
      sc = __builtin_amdgcn_mfma_f32_16x16x4f32(k.w, qq[dt].w, sc, 0, 0, 0);
    }
    return sc;
  };
  auto add_values = [&](int b, const gla_floatx4& sc) {
#pragma unroll
    for (int vt = 0; vt < VT; ++vt)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(sc[r], bf16_to_f32(L.v[(b * GLA_BLK + 4 * hi + r) * VS + vt * 16 + lo]),
                                                     o[vt], 0, 0, 0);
  };
  {
    gla_floatx4 sc = {0.f, 0.f, 0.f, 0.f};
    if (!L.thin[w]) {
      float4 qd[DT];
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const float4 g = *(const float4*)(L.G + w * DP + dt * 16 + 4 * hi);
        qd[dt] = make_float4(qf[dt].x * __builtin_amdgcn_rcpf(g.x), qf[dt].y * __builtin_amdgcn_rcpf(g.y),
                             qf[dt].z * __builtin_amdgcn_rcpf(g.z), qf[dt].w * __builtin_amdgcn_rcpf(g.w));
      }
      sc = scores(w, qd);
    } else {
      const int tq = w * GLA_BLK + lo;
      const bf16_t* qr = A.proj + (size_t)(n0 + (tq < n ? tq : 0)) * A.ld + A.q_off + h * A.D;
      for (int d = 0; d < A.D; ++d) {
        const float qv = bf16_to_f32(qr[d]) * A.q_scale, lq = L.la[tq * DS + d];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int tk = w * GLA_BLK + 4 * hi + r;
          const float kv = bf16_to_f32(A.proj[(size_t)(n0 + (tk < n ? tk : 0)) * A.ld + A.k_off + h * A.D + d]);
          sc[r] = fmaf(qv * kv, __builtin_amdgcn_exp2f(fminf(lq - L.la[tk * DS + d], 0.f)), sc[r]);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) sc[r] = 4 * hi + r <= lo ? sc[r] : 0.f;
    add_values(w, sc);
  }
  for (int b = w - 1; b >= 0; --b) {
    add_values(b, scores(b, qf));
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const float4 g = *(const float4*)(L.G + b * DP + dt * 16 + 4 * hi);
      qf[dt].x *= g.x; qf[dt].y *= g.y; qf[dt].z *= g.z; qf[dt].w *= g.w;
    }
  }
#pragma unroll
  for (int vt = 0; vt < VT; ++vt) {
    if (!EARLY) {
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) s0[0][dt] = start_piece(vt, dt);
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const float4 x = s0[EARLY ? vt : 0][dt];
      o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[dt].x, x.x, o[vt], 0, 0, 0);
      o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[dt].y, x.y, o[vt], 0, 0, 0);
      o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[dt].z, x.z, o[vt], 0, 0, 0);
      o[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[dt].w, x.w, o[vt], 0, 0, 0);
    }
  }
  // rows 4 hi + r: the read-out's norm, gain and gate
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    float ss = 0.f;
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) ss = fmaf(o[vt][r], o[vt][r], ss);
    const float inv = 1.0f / sqrtf(group_sum<16>(ss) / (float)A.Dv + A.eps);
    const int tok = w * GLA_BLK + 4 * hi + r;
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) {
      const int v = vt * 16 + lo;
      const float gt = bf16_to_f32(gate[vt][r]);
      const float g = gt * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-GLA_LOG2E * gt));
      if (tok < n && v < A.Dv) A.y[(size_t)(n0 + tok) * A.y_ld + h * A.Dv + v] = f32_to_bf16(o[vt][r] * inv * gain[vt] * g);
    }
  }
}

// 1 when da_gla_decode and da_gla_chunked take these sizes (state rows of `state_ld` floats)
extern "C" int da_gla_serve_takes(int D, int Dv, int state_ld) {
  return D > 0 && D % 4 == 0 && D <= GLA_SERVE_D && Dv > 0 && Dv <= GLA_SERVE_D && state_ld % 4 == 0;
}
// 1 when they work out the decays' arguments from a low rank of so many numbers
extern "C" int da_gla_low_takes(int rank) { return rank > 0 && rank % 4 == 0 && rank <= GLA_LOW_MAX; }

static int gla_serve_args(GlaServeArgs& A, const char* what, const void* proj, int ld, int q_off, int k_off, int v_off, int g_off,
                          int low_off, const void* up, int rank, const float* raw, int raw_ld, const float* bias, float tau,
                          float q_scale, const void* gain, int gain_dtype, float eps, float* state, long state_ld,
                          const int* state_slots, const int* q_start, void* y, int y_ld, int seq0, int n_seqs, int H, int D,
                          int Dv, int write) {
  DA_REQUIRE(seq0 >= 0 && n_seqs >= 0 && H > 0, "%s: bad sizes", what);
  DA_REQUIRE(da_gla_serve_takes(D, Dv, (int)(state_ld % 4)) && state_ld >= (long)H * Dv * D, "%s: head sizes %d and %d with state rows of %ld are not taken", what, D, Dv, state_ld);
  DA_REQUIRE((uintptr_t)state % 16 == 0 && (uintptr_t)up % 8 == 0, "%s: operands must be aligned", what);
  DA_REQUIRE(q_off >= 0 && k_off >= 0 && v_off >= 0 && g_off >= 0 && ld >= q_off + H * D && ld >= k_off + H * D &&
             ld >= v_off + H * Dv && ld >= g_off + H * Dv, "%s: q, k, v and gate leave the row", what);
  DA_REQUIRE((up != nullptr) != (raw != nullptr), "%s: the decays' arguments come as rows or from a low rank", what);
  DA_REQUIRE(!up || (da_gla_low_takes(rank) && low_off >= 0 && ld >= low_off + rank), "%s: a low rank of %d is not taken", what, rank);
  DA_REQUIRE(!raw || raw_ld >= H * D, "%s: the decays' rows are too short", what);
  DA_REQUIRE(y_ld >= H * Dv && tau > 0.f && eps > 0.f, "%s: bad output rows, tau or eps", what);
  A.proj = (const bf16_t*)proj; A.ld = ld; A.q_off = q_off; A.k_off = k_off; A.v_off = v_off; A.g_off = g_off; A.low_off = low_off;
  A.up = (const bf16_t*)up; A.rank = rank; A.raw = raw; A.raw_ld = raw_ld; A.bias = bias; A.gain = gain; A.gain_dtype = gain_dtype;
  A.state = state; A.state_ld = state_ld; A.state_slots = state_slots; A.q_start = q_start; A.y = (bf16_t*)y; A.y_ld = y_ld;
  A.H = H; A.D = D; A.Dv = Dv; A.write = write; A.seq0 = seq0; A.n_seqs = n_seqs; A.q_scale = q_scale; A.inv_tau = 1.0f / tau;
  const bool rows = ld % 4 == 0 && (uintptr_t)proj % 8 == 0;
  A.whole_qk = rows && q_off % 4 == 0 && k_off % 4 == 0;
  A.whole_v = rows && v_off % 4 == 0 && Dv % 4 == 0;
  A.whole_low = rows && low_off % 4 == 0;
  A.eps = eps; A.n_chunks = 0; A.ends = nullptr; A.chunk_decay = nullptr;
  return 0;
}

// Sequences seq0 .. seq0 + n_seqs - 1, which bring one token each (more are not looked at).
extern "C" int da_gla_decode(const void* proj, int ld, int q_off, int k_off, int v_off, int g_off, int low_off, const void* up,
                             int rank, const float* raw, int raw_ld, const float* bias, float tau, float q_scale,
                             const void* gain, int gain_dtype, float eps, float* state, long state_ld, const int* state_slots,
                             const int* q_start, void* y, int y_ld, int seq0, int n_seqs, int H, int D, int Dv, int write,
                             void* stream) {
  GlaServeArgs A;
  const int rc = gla_serve_args(A, "gla_decode", proj, ld, q_off, k_off, v_off, g_off, low_off, up, rank, raw, raw_ld, bias, tau,
                                q_scale, gain, gain_dtype, eps, state, state_ld, state_slots, q_start, y, y_ld, seq0, n_seqs, H, D,
                                Dv, write);
  if (rc || n_seqs == 0) return rc;
  DA_REQUIRE((long)n_seqs * H < (1L << 31), "gla_decode: too many sequences or heads for one launch");
  const dim3 grid((unsigned)(n_seqs * H)), block(256);
  if (D <= 64) hipLaunchKernelGGL(gla_decode_kernel<4>, grid, block, 0, (hipStream_t)stream, A);
  else hipLaunchKernelGGL(gla_decode_kernel<8>, grid, block, 0, (hipStream_t)stream, A);
  DA_CHECK_LAUNCH("gla_decode");
  return 0;
}

template <int DT, int VT>
static int gla_chunked_go(const GlaServeArgs& A, hipStream_t st) {
  const dim3 grid((unsigned)A.H, (unsigned)A.n_chunks, (unsigned)A.n_seqs), block(256);
  hipLaunchKernelGGL((gla_states_kernel<DT, VT>), grid, block, 0, st, A);
  DA_CHECK_LAUNCH("gla_states");
  const long n = (long)A.n_seqs * A.H * A.Dv * A.D;
  hipLaunchKernelGGL(gla_carry_kernel, dim3((unsigned)da_ceil_div(n, 256)), dim3(256), 0, st, A);
  DA_CHECK_LAUNCH("gla_carry");
  hipLaunchKernelGGL((gla_output_kernel<DT, VT>), grid, block, 0, st, A);
  DA_CHECK_LAUNCH("gla_output");
  return 0;
}

// Portions of any length: sequences seq0 .. seq0 + n_seqs - 1, of which the longest brings max_rows rows.  scratch: 32-bit,
// n_seqs * ceil(max_rows / 64) * H * D * (Dv + 1) floats.
extern "C" int da_gla_chunked(const void* proj, int ld, int q_off, int k_off, int v_off, int g_off, int low_off, const void* up,
                              int rank, const float* raw, int raw_ld, const float* bias, float tau, float q_scale,
                              const void* gain, int gain_dtype, float eps, float* state, long state_ld, const int* state_slots,
                              const int* q_start, void* y, int y_ld, int seq0, int n_seqs, int H, int D, int Dv, int write,
                              int max_rows, float* scratch, long scratch_floats, void* stream) {
  GlaServeArgs A;
  const int rc = gla_serve_args(A, "gla_chunked", proj, ld, q_off, k_off, v_off, g_off, low_off, up, rank, raw, raw_ld, bias, tau,
                                q_scale, gain, gain_dtype, eps, state, state_ld, state_slots, q_start, y, y_ld, seq0, n_seqs, H, D,
                                Dv, write);
  if (rc || n_seqs == 0) return rc;
  DA_REQUIRE(max_rows > 0, "gla_chunked: the longest portion has %d rows", max_rows);
  A.n_chunks = da_ceil_div(max_rows, GLA_CHUNK);
  const long per = (long)n_seqs * A.n_chunks * H * D;
  DA_REQUIRE(scratch != nullptr && (uintptr_t)scratch % 16 == 0 && scratch_floats >= per * (Dv + 1),
             "gla_chunked: a scratch of %ld floats is needed", per * (Dv + 1));
  DA_REQUIRE(n_seqs <= 65535 && A.n_chunks <= 65535, "gla_chunked: too many sequences or chunks for one launch");
  A.ends = scratch;
  A.chunk_decay = scratch + per * Dv;
  hipStream_t st = (hipStream_t)stream;
#define GLA_VALUES(N)                                        \
  do {                                                       \
    if (Dv <= 32) return gla_chunked_go<N, 2>(A, st);        \
    if (Dv <= 64) return gla_chunked_go<N, 4>(A, st);        \
    return gla_chunked_go<N, 8>(A, st);                      \
  } while (0)
  if (D <= 32) GLA_VALUES(2);
  if (D <= 64) GLA_VALUES(4);
  GLA_VALUES(8);
#undef GLA_VALUES
}
