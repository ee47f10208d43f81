// A linear recurrence with one real number of state a channel and a decay that the input sets.
//
//   u    = filter(x)                      per channel a short causal filter with a bias (the input x is a projection)
//   r, i = logistic(A_b u_b), logistic(I_b u_b)      block by block: u is cut into equal parts of `bs` channels
//   log a = rate[c] * r,  a = e^(log a)   rate = -strength * softplus(lam), worked out once per channel
//   S   <- a S + sqrt(1 - a^2) * i * u    all of it 32-bit; S = 0 at a sequence's start
//   out  = S * act(y)                     y: the other branch's projection
//
// A request's state is one 32-bit row [ S: C | the filter's last K - 1 inputs: (K - 1) x C, oldest first ].  A sequence
// without a slot (a padding row of a fixed-shape step) reads zeros and keeps nothing.
//
//   da_rglru_walk     from u and the square matrices' sums, token by token, a thread a channel; both dtypes, any sizes.
//                     The 32-bit path, and the reference of the other forms.
//   da_rglru_decode   one-token sequences, from the projections to out in one launch: a workgroup takes 16 sequences and
//                     a block of channels; filter (whose kept inputs move on), the block's two square matrices on the
//                     matrix cores, gates, state, branch.
//   da_rglru_portion  portions, in chunks of 32 tokens that run side by side.  A chunk of a block of channels: filter into
//                     LDS, the square matrices on the matrix cores (16x16x32; a lane's four results of a tile are four
//                     consecutive tokens of one channel), then the recurrence as a scan of pairs (product of the decays,
//                     state from zero): four tokens in a lane's registers, four lanes by two exchanges, the chunk's tiles
//                     one after the other.  A step whose portions all fit a chunk takes one launch; longer ones two:
//                     every chunk's pair, then every chunk again, with the pairs before it folded into its starting
//                     state (the second look at x and the matrices costs less than keeping two 32-bit numbers a token and
//                     channel).
//
// The order of a token's sums depends on its place in its portion and, for the fold, on its chunk's number only.
#include "gemm_common.h"

#define LRU_MAX_TAPS 16
#define LRU_TOK 32            // tokens of a chunk
#define LRU_MAX_BLOCK 256
#define LRU_LOG2E 1.4426950408889634f

// 1 - e^x for x <= 0: the series near zero, where the difference would cancel (`e` is e^x)
__device__ __forceinline__ float lru_one_minus_exp(float x, float e) {
  const float s = -x * (1.f + x * (1.f / 2) * (1.f + x * (1.f / 3) * (1.f + x * (1.f / 4) * (1.f + x * (1.f / 5) * (1.f + x * (1.f / 6) * (1.f + x * (1.f / 7)))))));
  return x > -0.35f ? s : 1.f - e;
}

__device__ __forceinline__ float lru_logistic(float z) {
  return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-LRU_LOG2E * z));
}

// the decay and what a token adds to the state, from the square matrices' sums (the hardware's exp2, reciprocal and root,
// each within a unit or two in the last place of 32 bits)
__device__ __forceinline__ void lru_step(float zr, float zi, float rate, float u, float& a, float& add) {
  const float la = rate * lru_logistic(zr);
  a = __builtin_amdgcn_exp2f(LRU_LOG2E * la);
  const float m2 = lru_one_minus_exp(2.f * la, a * a);
  const float root = m2 > 0.f ? m2 * __builtin_amdgcn_rsqf(m2) : 0.f;
  add = root * lru_logistic(zi) * u;
}

// ---- token by token -----------------------------------------------------------------------------------------------
template <typename T>
__global__ void rglru_walk_kernel(const T* __restrict__ u, int u_ld, const float* __restrict__ raw, int raw_ld, int bs,
                                  const float* __restrict__ rate, const T* __restrict__ y, int y_ld, int act,
                                  float* __restrict__ state, long state_ld, const int* __restrict__ state_slots,
                                  const int* __restrict__ q_start, T* __restrict__ out, int out_ld, int S, int C, int write) {
  const long t = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= (long)S * C) return;
  const int s = (int)(t / C), c = (int)(t % C);
  const int slot = state_slots[s];
  const int zr = c / bs * 2 * bs + c % bs;               // the block's sums: r's, then i's
  const float rt = rate[c];
  float st = slot >= 0 ? state[(size_t)slot * state_ld + c] : 0.f;
  for (int n = q_start[s]; n < q_start[s + 1]; ++n) {
    const float r = 1.f / (1.f + expf(-raw[(size_t)n * raw_ld + zr])), i = 1.f / (1.f + expf(-raw[(size_t)n * raw_ld + zr + bs]));
    const float la = rt * r;
    st = expf(la) * st + sqrtf(-expm1f(2.f * la)) * i * to_f32(u[(size_t)n * u_ld + c]);
    from_f32(&out[(size_t)n * out_ld + c], st * apply_act(to_f32(y[(size_t)n * y_ld + c]), act));
  }
  if (write && slot >= 0) state[(size_t)slot * state_ld + c] = st;
}

extern "C" int da_rglru_walk(const void* u, int dtype, int u_ld, const float* raw, int raw_ld, int bs, const float* rate,
                             const void* y, int y_ld, int act, float* state, long state_ld, const int* state_slots,
                             const int* q_start, void* out, int out_ld, int S, int C, int write, void* stream) {
  DA_REQUIRE(S >= 0 && C > 0 && bs > 0 && C % bs == 0, "rglru_walk: %d channels in blocks of %d", C, bs);
  DA_REQUIRE(u_ld >= C && raw_ld >= 2 * C && y_ld >= C && out_ld >= C && state_ld >= C, "rglru_walk: rows too short");
  DA_REQUIRE(act >= DA_ACT_NONE && act < DA_ACT_GLU_CAPPED, "rglru_walk: unknown activation %d", act);
  if (S == 0) return 0;
  const dim3 grid(da_ceil_div((long)S * C, 64));
  if (dtype == DA_BF16)
    hipLaunchKernelGGL(rglru_walk_kernel<bf16_t>, grid, dim3(64), 0, (hipStream_t)stream, (const bf16_t*)u, u_ld, raw, raw_ld,
                       bs, rate, (const bf16_t*)y, y_ld, act, state, state_ld, state_slots, q_start, (bf16_t*)out, out_ld, S, C, write);
  else
    hipLaunchKernelGGL(rglru_walk_kernel<float>, grid, dim3(64), 0, (hipStream_t)stream, (const float*)u, u_ld, raw, raw_ld,
                       bs, rate, (const float*)y, y_ld, act, state, state_ld, state_slots, q_start, (float*)out, out_ld, S, C, write);
  DA_CHECK_LAUNCH("rglru_walk");
  return 0;
}

// ---- serving in bfloat16 --------------------------------------------------------------------------------------------
// What the serving kernels read of a layer and a step.  Rows of yx are [ y: C | x: C ].
struct LruIn {
  const bf16_t* yx; int ld;
  const float* conv_w;        // [K][C], the last row meets the token itself
  const float* conv_b;        // [C]
  const bf16_t* gate_w;       // [blocks][2 bs][bs]: r's rows, then i's
  const float* gate_b;        // [blocks][2 bs]
  const float* rate;          // [C]
  float* state; long state_ld;
  const int* slots;
  const int* q_start;
  bf16_t* out; int out_ld;
  int C, bs, K, act, write;
};

__device__ __forceinline__ void lru_unpack8(uint4 v, float* f) {
  const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    f[2 * e] = __uint_as_float(w[e] << 16);
    f[2 * e + 1] = __uint_as_float(w[e] & 0xffff0000u);
  }
}
__device__ __forceinline__ uint4 lru_pack8(const float* f) {
  return make_uint4(pack2_bf16(f[0], f[1]), pack2_bf16(f[2], f[3]), pack2_bf16(f[4], f[5]), pack2_bf16(f[6], f[7]));
}
__device__ __forceinline__ void lru_load8(const float* p, float* f) {
  const float4 a = *(const float4*)p, b = *(const float4*)(p + 4);
  f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
}
__device__ __forceinline__ void lru_store8(float* p, const float* f) {
  *(float4*)p = make_float4(f[0], f[1], f[2], f[3]);
  *(float4*)(p + 4) = make_float4(f[4], f[5], f[6], f[7]);
}

// A pair (product of decays, state from zero) a lane; the four lanes of a channel (16 apart) hold pieces of time in order.
// Afterwards a lane's pair is that of everything up to its own piece.
__device__ __forceinline__ void lru_fold_lanes(int lane, int g, float& p, float& s) {
#pragma unroll
  for (int back = 16; back <= 32; back *= 2) {
    const int from = lane - back >= 0 ? lane - back : lane;
    const float bp = __shfl(p, from, DA_WAVE), bs = __shfl(s, from, DA_WAVE);
    if (16 * g >= back) { s = p * bs + s; p = p * bp; }
  }
}

// KS: pieces of 32 along a block's channels; a wavefront owns 16 channels, its two matrices' rows in registers.
template <int KS>
__device__ __forceinline__ void lru_load_gates(const LruIn& in, int b, int n0, int lane, uint4 (&wr)[KS], uint4 (&wi)[KS]) {
  const int fr = lane % 16, fk = (lane / 16) * 8;
  const int row = n0 + fr < in.bs ? n0 + fr : 0;
  const bf16_t* w = in.gate_w + ((size_t)b * 2 * in.bs + row) * in.bs;
#pragma unroll
  for (int k = 0; k < KS; ++k) {
    const int kk = k * 32 + fk < in.bs ? k * 32 + fk : 0;          // (past the block: met by zeros in u)
    wr[k] = load16(w + kk);
    wi[k] = load16(w + (size_t)in.bs * in.bs + kk);
  }
}

// Decode: sequence j of the first n has row j (one-token sequences lead a step).  blockDim = 2 KS wavefronts, so that every 16 channels have one.
// KT: taps rounded up; taps that do not exist have no weight and read the token itself.
template <int KS, int KT>
__global__ void __launch_bounds__(2 * KS * DA_WAVE)
rglru_decode_kernel(LruIn in, int n) {
  constexpr int PITCH = KS * 32 + 8;
  __shared__ __attribute__((aligned(16))) bf16_t us[16][PITCH];
  const int b = blockIdx.x, j0 = blockIdx.y * 16;
  const int t = threadIdx.x, lane = t % DA_WAVE, wave = t / DA_WAVE;
  const int fr = lane % 16, g = lane / 16;
  const int c0 = b * in.bs, n0 = wave * 16;
  const bool cols = n0 < in.bs;                                     // (the same for the wavefront)
  const int ch = n0 + fr < in.bs ? n0 + fr : 0, c = c0 + ch;
  uint4 wr[KS], wi[KS];
  if (cols) lru_load_gates<KS>(in, b, n0, lane, wr, wi);
  // this lane's four sequences: state, branch, what the gates need
  float s_old[4], yv[4];
  int slot[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int j = j0 + 4 * g + r, jj = j < n ? j : n - 1;
    slot[r] = in.slots[jj];
    yv[r] = bf16_to_f32(in.yx[(size_t)jj * in.ld + c]);
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) s_old[r] = in.state[(size_t)(slot[r] >= 0 ? slot[r] : 0) * in.state_ld + c];
  const float br = in.gate_b[(size_t)b * 2 * in.bs + ch], bi = in.gate_b[(size_t)b * 2 * in.bs + in.bs + ch], rate = in.rate[c];
  // the filter: 8 channels of a sequence a thread, which also moves the kept inputs on
  for (int e = t; e < 16 * KS * 4; e += 2 * KS * DA_WAVE) {
    const int j = e / (KS * 4), c8 = (e % (KS * 4)) * 8;
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (c8 < in.bs && j0 + j < n) {
      const int sl = in.slots[j0 + j];
      float xv[8], tail[KT - 1][8], w[KT][8];
      lru_unpack8(load16(in.yx + (size_t)(j0 + j) * in.ld + in.C + c0 + c8), xv);
      float* tp = in.state + (size_t)(sl >= 0 ? sl : 0) * in.state_ld + in.C + c0 + c8;
#pragma unroll
      for (int k = 0; k < KT - 1; ++k) lru_load8(k < in.K - 1 ? tp + (size_t)k * in.C : tp - in.C, tail[k]);   // (or the row's S)
#pragma unroll
      for (int k = 0; k < KT; ++k) lru_load8(in.conv_w + (size_t)(k < in.K ? k : 0) * in.C + c0 + c8, w[k]);
      lru_load8(in.conv_b + c0 + c8, acc);
#pragma unroll
      for (int k = 0; k < KT - 1; ++k)
#pragma unroll
        for (int q = 0; q < 8; ++q)
          if (k < in.K - 1 && sl >= 0) acc[q] = fmaf(w[k][q], tail[k][q], acc[q]);
#pragma unroll
      for (int k = 0; k < KT; ++k)
        if (k == in.K - 1) {
#pragma unroll
          for (int q = 0; q < 8; ++q) acc[q] = fmaf(w[k][q], xv[q], acc[q]);
        }
      if (in.write && sl >= 0) {
#pragma unroll
        for (int k = 0; k < KT - 1; ++k) {
          if (k < in.K - 2) lru_store8(tp + (size_t)k * in.C, tail[k + 1 < KT - 1 ? k + 1 : k]);
          else if (k == in.K - 2) lru_store8(tp + (size_t)k * in.C, xv);
        }
      }
    }
    *(uint4*)&us[j][c8] = lru_pack8(acc);
  }
  __syncthreads();
  if (!cols) return;
  floatx4 ar = {0.f, 0.f, 0.f, 0.f}, ai = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int k = 0; k < KS; ++k) {
    const bf16x8_t a = __builtin_bit_cast(bf16x8_t, *(const uint4*)&us[fr][k * 32 + g * 8]);
    ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, __builtin_bit_cast(bf16x8_t, wr[k]), ar, 0, 0, 0);
    ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, __builtin_bit_cast(bf16x8_t, wi[k]), ai, 0, 0, 0);
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int j = 4 * g + r;
    if (j0 + j >= n || n0 + fr >= in.bs) continue;
    float a, add;
    lru_step(ar[r] + br, ai[r] + bi, rate, bf16_to_f32(us[j][ch]), a, add);
    const float st = a * (slot[r] >= 0 ? s_old[r] : 0.f) + add;
    if (in.write && slot[r] >= 0) in.state[(size_t)slot[r] * in.state_ld + c] = st;
    in.out[(size_t)(j0 + j) * in.out_ld + c] = f32_to_bf16(st * apply_act_bf16(yv[r], in.act));
  }
}

#define LRU_WHOLE 0     // portions of one chunk: state from and to the slot
#define LRU_PAIRS 1     // a chunk's pair (product of its decays, its state from zero) into `ends`
#define LRU_AGAIN 2     // a chunk from its starting state
#define LRU_FOLD 8      // pairs that a lane asks for at once

// Workgroup (block of channels and 64 of them, chunk, portion); wavefront w owns 16 channels.  ends: [portion][chunk][2][C].
// old: [portion][K][C], what the slots held before the step (state, then kept inputs; zeros without a slot): the first
// chunks of LRU_PAIRS write it down, LRU_AGAIN reads it, and its last chunks write the slots.
template <int KS, int KT, int MODE>
__global__ void __launch_bounds__(4 * DA_WAVE)
rglru_chunk_kernel(LruIn in, int seq0, int parts, float* __restrict__ ends, int max_chunks, float* __restrict__ old) {
  constexpr int PITCH = KS * 32 + 8, YP = 64 + 8;
  __shared__ __attribute__((aligned(16))) bf16_t us[LRU_TOK][PITCH];
  __shared__ __attribute__((aligned(16))) bf16_t ys[MODE == LRU_PAIRS ? 1 : LRU_TOK][YP];
  const int b = blockIdx.x / parts, part = blockIdx.x % parts, chunk = blockIdx.y, s = seq0 + blockIdx.z;
  const int first = in.q_start[s], len = in.q_start[s + 1] - first, t0 = chunk * LRU_TOK;
  if (t0 >= len) return;                                            // (the whole workgroup)
  const int slot = in.slots[s];
  const int nt = len - t0 < LRU_TOK ? len - t0 : LRU_TOK;
  const int t = threadIdx.x, lane = t % DA_WAVE, wave = t / DA_WAVE;
  const int fr = lane % 16, g = lane / 16;
  const int c0 = b * in.bs, n0 = part * 64 + wave * 16;
  const bool cols = n0 < in.bs;
  const int ch = n0 + fr < in.bs ? n0 + fr : 0, c = c0 + ch;
  uint4 wr[KS], wi[KS];
  if (cols) lru_load_gates<KS>(in, b, n0, lane, wr, wi);
  const float br = in.gate_b[(size_t)b * 2 * in.bs + ch], bi = in.gate_b[(size_t)b * 2 * in.bs + in.bs + ch], rate = in.rate[c];
  float* const row = in.state + (size_t)(slot >= 0 ? slot : 0) * in.state_ld;
  float* const was = MODE == LRU_WHOLE ? nullptr : old + (size_t)blockIdx.z * in.K * in.C;
  const float* tail = MODE == LRU_AGAIN ? was + in.C : (slot >= 0 ? row + in.C : nullptr);
  float start = 0.f;
  if (MODE == LRU_WHOLE) start = slot >= 0 ? row[c] : 0.f;
  if (MODE == LRU_AGAIN) start = was[c];
  // the pairs of the chunks before this one: a quarter of them, in a row, a group of 16 lanes; the first ones are asked
  // for here (chunks that are not there read the first and count as nothing)
  const float* const before = ends + (size_t)blockIdx.z * max_chunks * 2 * in.C + c;
  const int per = (chunk + 3) / 4, k_first = g * per, k_end = k_first + per < chunk ? k_first + per : chunk;
  float fp[LRU_FOLD], fs[LRU_FOLD];
  auto ask = [&](int k0) {
#pragma unroll
    for (int q = 0; q < LRU_FOLD; ++q) {
      const int k = k0 + q < k_end ? k0 + q : 0;
      fp[q] = before[(size_t)k * 2 * in.C];
      fs[q] = before[(size_t)k * 2 * in.C + in.C];
    }
  };
  if (MODE == LRU_AGAIN && chunk > 0) ask(k_first);
  if (MODE == LRU_PAIRS && chunk == 0) {
    for (int e = t; e < 64 * in.K; e += 4 * DA_WAVE) {
      const int k = e / 64, q = part * 64 + e % 64;
      if (q < in.bs) was[(size_t)k * in.C + c0 + q] = slot >= 0 ? row[(size_t)k * in.C + c0 + q] : 0.f;
    }
  }
  if (MODE != LRU_PAIRS) {
    // the branch's entries of this workgroup's 64 channels, 16 bytes a thread
    for (int e = t; e < LRU_TOK * 8; e += 4 * DA_WAVE) {
      const int tok = e / 8, cc = part * 64 + (e % 8) * 8;
      const uint4 v = load16(in.yx + (size_t)(first + t0 + (tok < nt ? tok : nt - 1)) * in.ld + c0 + (cc < in.bs ? cc : 0));
      *(uint4*)&ys[tok][(e % 8) * 8] = v;
    }
  }
  // the filter: 8 channels of a token a thread
  for (int e = t; e < LRU_TOK * KS * 4; e += 4 * DA_WAVE) {
    const int tok = e / (KS * 4), c8 = (e % (KS * 4)) * 8;
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (c8 < in.bs && tok < nt) {
      const int at = t0 + tok;                                      // the token's place in its portion
      uint4 xr[KT];
      float w[KT][8];
#pragma unroll
      for (int k = 0; k < KT; ++k) {                                // k: how many tokens back
        const int rr = k < in.K && at - k >= 0 ? at - k : at;
        xr[k] = load16(in.yx + (size_t)(first + rr) * in.ld + in.C + c0 + c8);
        lru_load8(in.conv_w + (size_t)(k < in.K ? in.K - 1 - k : 0) * in.C + c0 + c8, w[k]);
      }
      lru_load8(in.conv_b + c0 + c8, acc);
#pragma unroll
      for (int k = KT - 1; k >= 0; --k) {
        if (k >= in.K) continue;
        float v[8];
        lru_unpack8(xr[k], v);
        if (at - k < 0) {                                           // before the portion (its first rows only)
          if (tail) lru_load8(tail + (size_t)(in.K - 1 + at - k) * in.C + c0 + c8, v);
          else
#pragma unroll
            for (int q = 0; q < 8; ++q) v[q] = 0.f;
        }
#pragma unroll
        for (int q = 0; q < 8; ++q) acc[q] = fmaf(w[k][q], v[q], acc[q]);
      }
    }
    *(uint4*)&us[tok][c8] = lru_pack8(acc);
  }
  __syncthreads();
  if ((MODE == LRU_WHOLE || (MODE == LRU_AGAIN && t0 + LRU_TOK >= len)) && in.write && slot >= 0) {
    // the kept inputs after the step, a channel of this workgroup's a thread, the ones that stay moved on in ascending
    // order (with the slot itself as their source every read of the old ones lies before the barrier, and nobody else
    // reads these channels')
    for (int q = part * 64 + t; q < in.bs && q < part * 64 + 64; q += 4 * DA_WAVE)
      for (int k = 0; k < in.K - 1; ++k) {
        const int r = len - (in.K - 1) + k;
        row[(size_t)(k + 1) * in.C + c0 + q] = r >= 0 ? bf16_to_f32(in.yx[(size_t)(first + r) * in.ld + in.C + c0 + q])
                                                      : tail[(size_t)(in.K - 1 + r) * in.C + c0 + q];
      }
  }
  if (cols) {
    if (MODE == LRU_AGAIN && chunk > 0) {
      float ip = 1.f, is = 0.f;
      for (int k0 = k_first;;) {
#pragma unroll
        for (int q = 0; q < LRU_FOLD; ++q)
          if (k0 + q < k_end) {
            is = fp[q] * is + fs[q];
            ip = ip * fp[q];
          }
        k0 += LRU_FOLD;
        if (k0 - k_first >= per) break;                             // (the same for the wavefront)
        ask(k0);
      }
      lru_fold_lanes(lane, g, ip, is);
      start = __shfl(ip, 48 + fr, DA_WAVE) * start + __shfl(is, 48 + fr, DA_WAVE);
    }
    float run_p = 1.f, run_s = start;                               // everything before the tile: decays' product, state
#pragma unroll
    for (int i = 0; i < LRU_TOK / 16; ++i) {
      if (i * 16 >= nt) break;                                      // (the same for the workgroup)
      floatx4 ar = {0.f, 0.f, 0.f, 0.f}, ai = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        const bf16x8_t a = __builtin_bit_cast(bf16x8_t, *(const uint4*)&us[i * 16 + fr][k * 32 + g * 8]);
        ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, __builtin_bit_cast(bf16x8_t, wr[k]), ar, 0, 0, 0);
        ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, __builtin_bit_cast(bf16x8_t, wi[k]), ai, 0, 0, 0);
      }
      float p[4], st[4];                                            // up to token r of this lane's four, from zero
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tok = i * 16 + 4 * g + r;
        float a, add;
        lru_step(ar[r] + br, ai[r] + bi, rate, bf16_to_f32(us[tok][ch]), a, add);
        if (tok >= nt) { a = 1.f; add = 0.f; }
        p[r] = r ? p[r ? r - 1 : 0] * a : a;
        st[r] = r ? a * st[r ? r - 1 : 0] + add : add;
      }
      // with the lanes before this one that hold earlier tokens of the channel
      float ip = p[3], is = st[3];
      lru_fold_lanes(lane, g, ip, is);
      float ep = __shfl(ip, lane - 16 >= 0 ? lane - 16 : lane, DA_WAVE), es = __shfl(is, lane - 16 >= 0 ? lane - 16 : lane, DA_WAVE);
      if (g == 0) { ep = 1.f; es = 0.f; }
      const float in_s = ep * run_s + es;                           // the state in front of this lane's first token
      if (MODE != LRU_PAIRS) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int tok = i * 16 + 4 * g + r, yc = wave * 16 + fr;
          const float sv = p[r] * in_s + st[r];
          ys[tok][yc] = f32_to_bf16(sv * apply_act_bf16(bf16_to_f32(ys[tok][yc]), in.act));
        }
      }
      const float lp = __shfl(ip, 48 + fr, DA_WAVE), ls = __shfl(is, 48 + fr, DA_WAVE);        // the whole tile
      run_s = lp * run_s + ls;
      run_p = run_p * lp;
    }
    if (g == 0 && n0 + fr < in.bs) {
      if (MODE == LRU_PAIRS) {
        float* pair = ends + (((size_t)blockIdx.z * max_chunks + chunk) * 2) * in.C + c;
        pair[0] = run_p;
        pair[in.C] = run_s;
      } else if (t0 + LRU_TOK >= len && in.write && slot >= 0) {
        row[c] = run_s;
      }
    }
  }
  if (MODE != LRU_PAIRS) {
    __syncthreads();
    for (int e = t; e < nt * 8; e += 4 * DA_WAVE) {
      const int tok = e / 8, cc = part * 64 + (e % 8) * 8;
      if (cc < in.bs) *(uint4*)(in.out + (size_t)(first + t0 + tok) * in.out_ld + c0 + cc) = *(const uint4*)&ys[tok][(e % 8) * 8];
    }
  }
}

// 1 when the serving kernels take blocks of so many channels
extern "C" int da_rglru_serve_takes(int bs) { return bs > 0 && bs % 8 == 0 && bs <= LRU_MAX_BLOCK; }

static int lru_checks(const LruIn& in, const char* name) {
  DA_REQUIRE(da_rglru_serve_takes(in.bs) && in.C > 0 && in.C % in.bs == 0, "%s: %d channels in blocks of %d are not taken", name, in.C, in.bs);
  DA_REQUIRE(in.K >= 1 && in.K <= LRU_MAX_TAPS, "%s: %d taps (1 to %d are taken)", name, in.K, LRU_MAX_TAPS);
  DA_REQUIRE(in.ld >= 2 * in.C && in.ld % 8 == 0 && in.out_ld >= in.C && in.out_ld % 8 == 0 && in.state_ld >= (long)in.K * in.C && in.state_ld % 4 == 0,
             "%s: row lengths", name);
  DA_REQUIRE((uintptr_t)in.yx % 16 == 0 && (uintptr_t)in.conv_w % 16 == 0 && (uintptr_t)in.conv_b % 16 == 0 && (uintptr_t)in.gate_w % 16 == 0 &&
             (uintptr_t)in.state % 16 == 0 && (uintptr_t)in.out % 16 == 0, "%s: operands must be 16-byte aligned", name);
  DA_REQUIRE(in.act >= DA_ACT_NONE && in.act < DA_ACT_GLU_CAPPED, "%s: unknown activation %d", name, in.act);
  return 0;
}

#define LRU_PICK(GO)                                                   \
  do {                                                                 \
    if (in.bs <= 32) { if (in.K <= 4) GO(1, 4); else GO(1, 16); }      \
    else if (in.bs <= 64) { if (in.K <= 4) GO(2, 4); else GO(2, 16); } \
    else if (in.bs <= 128) { if (in.K <= 4) GO(4, 4); else GO(4, 16); } \
    else { if (in.K <= 4) GO(8, 4); else GO(8, 16); }                  \
  } while (0)

// The step's first n sequences, which bring one token each: sequence j has row j.
extern "C" int da_rglru_decode(const void* yx, int ld, const float* conv_w, const float* conv_b, const void* gate_w,
                               const float* gate_b, const float* rate, int act, float* state, long state_ld,
                               const int* state_slots, void* out, int out_ld, int n, int C, int bs, int K,
                               int write, void* stream) {
  const LruIn in{(const bf16_t*)yx, ld, conv_w, conv_b, (const bf16_t*)gate_w, gate_b, rate, state, state_ld, state_slots, nullptr,
                 (bf16_t*)out, out_ld, C, bs, K, act, write};
  if (lru_checks(in, "rglru_decode")) return 1;
  DA_REQUIRE(n >= 0, "rglru_decode: bad sizes");
  if (n == 0) return 0;
  const dim3 grid(C / bs, da_ceil_div(n, 16));
#define LRU_GO(KS, KT) hipLaunchKernelGGL((rglru_decode_kernel<KS, KT>), grid, dim3(2 * KS * DA_WAVE), 0, (hipStream_t)stream, in, n)
  LRU_PICK(LRU_GO);
#undef LRU_GO
  DA_CHECK_LAUNCH("rglru_decode");
  return 0;
}

extern "C" int da_rglru_chunk_tokens() { return LRU_TOK; }

// Sequences seq0 .. seq0 + S - 1 of the step, the longest of which brings max_len tokens.  scratch (when max_len is more
// than a chunk, or a block has more than 64 channels): S * (chunks * 2 + K) * C floats.
extern "C" int da_rglru_portion(const void* yx, int ld, const float* conv_w, const float* conv_b, const void* gate_w,
                                const float* gate_b, const float* rate, int act, float* state, long state_ld,
                                const int* state_slots, const int* q_start, void* out, int out_ld, int seq0, int S, int C, int bs,
                                int K, int write, int max_len, float* scratch, long scratch_floats, void* stream) {
  const LruIn in{(const bf16_t*)yx, ld, conv_w, conv_b, (const bf16_t*)gate_w, gate_b, rate, state, state_ld, state_slots, q_start,
                 (bf16_t*)out, out_ld, C, bs, K, act, write};
  if (lru_checks(in, "rglru_portion")) return 1;
  DA_REQUIRE(seq0 >= 0 && S >= 0 && max_len >= 0, "rglru_portion: bad sizes");
  if (S == 0 || max_len == 0) return 0;
  const int chunks = da_ceil_div(max_len, LRU_TOK), parts = da_ceil_div(bs, 64);
  DA_REQUIRE(S <= 65535 && chunks <= 65535, "rglru_portion: too many portions or chunks for one launch");
  hipStream_t st = (hipStream_t)stream;
  const dim3 grid(C / bs * parts, chunks, S), block(4 * DA_WAVE);
  if (chunks == 1 && parts == 1) {
#define LRU_GO(KS, KT) hipLaunchKernelGGL((rglru_chunk_kernel<KS, KT, LRU_WHOLE>), grid, block, 0, st, in, seq0, parts, nullptr, 1, nullptr)
    LRU_PICK(LRU_GO);
#undef LRU_GO
    DA_CHECK_LAUNCH("rglru_portion");
    return 0;
  }
  const long need = (long)S * (2L * chunks + K) * C;
  DA_REQUIRE(scratch && scratch_floats >= need, "rglru_portion: the scratch holds %ld numbers, %ld are needed", scratch_floats, need);
  float* old = scratch + (long)S * chunks * 2 * C;
#define LRU_GO(KS, KT)                                                                                                          \
  do {                                                                                                                          \
    hipLaunchKernelGGL((rglru_chunk_kernel<KS, KT, LRU_PAIRS>), grid, block, 0, st, in, seq0, parts, scratch, chunks, old);     \
    hipLaunchKernelGGL((rglru_chunk_kernel<KS, KT, LRU_AGAIN>), grid, block, 0, st, in, seq0, parts, scratch, chunks, old);     \
  } while (0)
  LRU_PICK(LRU_GO);
#undef LRU_GO
  DA_CHECK_LAUNCH("rglru_portion");
  return 0;
}
