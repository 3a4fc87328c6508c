// A state-space recurrence with one decay a head and token (structured state-space duality): a
// matrix S [N, dv] a head in 32-bit,
//
//   dt_t = softplus(s_t + b),   S_t = exp(-exp(A) dt_t) S_(t-1) + dt_t B_t x_t^T,
//   y_t  = S_t^T C_t + D x_t
//
// with x [dv] a head, and B and C [N] shared by the H / G neighbouring heads of a group.
//
//  * state_space_walk    token by token, every size, both storage types, all 32-bit: single tokens,
//                        short portions and the whole 32-bit path
//  * state_space_chunks  bfloat16 rows, portions in chunks of 128 tokens side by side.  With l_t =
//                        -exp(A) dt_t, L_i its sum over a chunk's tokens 0 .. i, S the state before
//                        the chunk:
//                          y_i = exp(L_i) S^T C_i + sum_j<=i exp(L_i - L_j) dt_j (C_i . B_j) x_j + D x_i
//                          S  <- exp(L_n) S + sum_j exp(L_n - L_j) dt_j B_j x_j^T
//                        which are matrix products: (1) every chunk's own sum, (2) the states at the
//                        chunks' starts one after the other, (3) every chunk's outputs.  The
//                        products run in bfloat16 MFMAs with 32-bit sums.  x, B and C are bfloat16
//                        rows; an operand that is a 32-bit number (the weighted x, the weights of
//                        the second sum, the state) enters as the sum of two bfloat16 numbers, its
//                        rounding and the rounding of what that leaves (2^-16 relative).  Only
//                        differences of L enter an exponential, all of them at most 0.
//
// A request's state is laid out [head][value column][channels padded to 4].
#include "zf_chunks.h"

struct StateSpace {
  const float* steps;          // s [T, H], float32
  const float* a_log;          // A [H]
  const float* bias;           // b [H]
  const float* skip;           // D [H]
  int H, G, N, dv, NP;         // NP: N padded to 4
  // single tokens, bfloat16: steps null, s_h = w_h . h instead, formed where it is used (h [T, K],
  // w [H, K], K a multiple of 8, rows on 16 bytes)
  const bf16_t* h;
  const bf16_t* w;
  int K;
};

// 8 neighbouring products of w . h
__device__ __forceinline__ float ss_dot8(const uint4& x, const uint4& y, float a) {
  const uint32_t xs[4] = {x.x, x.y, x.z, x.w}, ys[4] = {y.x, y.y, y.z, y.w};
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    a = fmaf(__uint_as_float(xs[e] << 16), __uint_as_float(ys[e] << 16), a);
    a = fmaf(__uint_as_float(xs[e] & 0xffff0000u), __uint_as_float(ys[e] & 0xffff0000u), a);
  }
  return a;
}

__device__ __forceinline__ float ss_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// ---------------------------------------------------------------- token by token
// grid (sequence, head, block of value columns); a wave's lanes hold LPC lanes of 4 channels for
// each of 64 / LPC value columns side by side, SS_NC such groups of columns one behind the other.
// Eight tokens' rows at a time lie in LDS as floats.  A column's partial outputs
// are added over its lanes in an order that depends on LPC alone.
#define SS_NC 4
#define SS_TC 8

template <typename T, int LPC>
__global__ __launch_bounds__(256) void state_space_walk_kernel(
    const T* __restrict__ xr, long long x_stride, const T* __restrict__ br, const T* __restrict__ cr,
    long long bc_stride, StateSpace p, float* __restrict__ state, long long slot_stride,
    const int* __restrict__ state_slots, const int* __restrict__ q_start,
    const int* __restrict__ seqs, float* __restrict__ out) {
  constexpr int CPW = ZF_WAVE / LPC;                 // columns side by side in a wave
  constexpr int KW = 4 * LPC;
  constexpr int VBMAX = 4 * SS_NC * CPW;
  __shared__ __attribute__((aligned(16))) float bs[SS_TC * KW], cs[SS_TC * KW];
  __shared__ float xs[SS_TC * VBMAX];
  __shared__ float gs[SS_TC], red[16];
  const int s = seqs != nullptr ? seqs[blockIdx.x] : blockIdx.x;
  const int hd = blockIdx.y, grp = hd / (p.H / p.G);
  const int t0 = q_start[s], t1 = q_start[s + 1];
  const int tid = threadIdx.x, wave = tid / ZF_WAVE, lane = tid % ZF_WAVE;
  const int VB = (blockDim.x / ZF_WAVE) * SS_NC * CPW;
  const int v0 = blockIdx.z * VB;
  const int cg = lane % LPC, cl = lane / LPC;
  const bool live = 4 * cg < p.NP;
  float* st = state + (size_t)state_slots[s] * slot_stride + (size_t)hd * p.dv * p.NP;
  // a single token: its rows, and what its step size is the product of, are asked for ahead of the
  // matrix (which takes longest to come)
  const bool own = p.h != nullptr;                   // (then every sequence brings one token)
  const bool one = t1 - t0 == 1 && KW <= (int)blockDim.x && VB <= (int)blockDim.x;
  float b1 = 0.f, c1 = 0.f, x1 = 0.f, s1 = 0.f;
  constexpr int DOTS = 2;
  uint4 hv[DOTS], wv[DOTS];
  const bf16_t* hrow = p.h + (size_t)t0 * p.K;
  const bf16_t* wrow = p.w + (size_t)hd * p.K;
  if (one) {
    if (tid < p.N) {
      const size_t at = (size_t)t0 * bc_stride + (size_t)grp * p.N + tid;
      b1 = load_as_float<T>(br + at);
      c1 = load_as_float<T>(cr + at);
    }
    if (tid < VB && v0 + tid < p.dv)
      x1 = load_as_float<T>(xr + (size_t)t0 * x_stride + (size_t)hd * p.dv + v0 + tid);
    if (!own) s1 = p.steps[(size_t)t0 * p.H + hd];
  }
  if (own && t0 < t1) {
#pragma unroll
    for (int u = 0; u < DOTS; ++u) {
      const int i = (tid + u * blockDim.x) * 8;
      hv[u] = wv[u] = make_uint4(0u, 0u, 0u, 0u);
      if (i < p.K) {
        hv[u] = *(const uint4*)(hrow + i);
        wv[u] = *(const uint4*)(wrow + i);
      }
    }
  }
  float4 S[SS_NC];
  int col[SS_NC];
#pragma unroll
  for (int i = 0; i < SS_NC; ++i) {
    col[i] = (wave * SS_NC + i) * CPW + cl;          // within the block
    S[i] = float4{0.f, 0.f, 0.f, 0.f};
    if (live && v0 + col[i] < p.dv)
      S[i] = *(const float4*)(st + (size_t)(v0 + col[i]) * p.NP + 4 * cg);
  }
  const float rate = expf(p.a_log[hd]), bias = p.bias[hd], skip = p.skip[hd];
  if (own && t0 < t1) {
    float a = 0.f;
#pragma unroll
    for (int u = 0; u < DOTS; ++u) a = ss_dot8(hv[u], wv[u], a);
    for (int i = (tid + DOTS * blockDim.x) * 8; i < p.K; i += blockDim.x * 8)
      a = ss_dot8(*(const uint4*)(hrow + i), *(const uint4*)(wrow + i), a);
    s1 = block_sum(a, red);
  }
  auto step_size = [&](int t) {
    return ss_softplus((own || one ? s1 : p.steps[(size_t)t * p.H + hd]) + bias);
  };
  for (int tc = t0; tc < t1; tc += SS_TC) {
    const int n = min(SS_TC, t1 - tc);
    __syncthreads();                                 // the rows before are done with
    if (one) {
      const float dt = step_size(t0);
      if (tid < KW) {
        bs[tid] = dt * b1;
        cs[tid] = c1;
      }
      if (tid < VB) xs[tid] = x1;
    } else {
      for (int i = tid; i < n * KW; i += blockDim.x) {
        const int t = i / KW, c = i % KW;
        float bv = 0.f, cv = 0.f;
        if (c < p.N) {
          const size_t at = (size_t)(tc + t) * bc_stride + (size_t)grp * p.N + c;
          bv = step_size(tc + t) * load_as_float<T>(br + at);
          cv = load_as_float<T>(cr + at);
        }
        bs[i] = bv;
        cs[i] = cv;
      }
      for (int i = tid; i < n * VB; i += blockDim.x) {
        const int t = i / VB, x = i % VB;
        xs[t * VBMAX + x] = v0 + x < p.dv
            ? load_as_float<T>(xr + (size_t)(tc + t) * x_stride + (size_t)hd * p.dv + v0 + x) : 0.f;
      }
    }
    if (tid < n) gs[tid] = expf(-(rate * step_size(tc + tid)));
    __syncthreads();
    for (int t = 0; t < n; ++t) {
      const float4 b4 = *(const float4*)(bs + t * KW + 4 * cg);
      const float4 c4 = *(const float4*)(cs + t * KW + 4 * cg);
      const float g = gs[t];
      float r4[SS_NC];
#pragma unroll
      for (int i = 0; i < SS_NC; ++i) {
        const float xv = xs[t * VBMAX + col[i]];
        S[i].x = fmaf(g, S[i].x, b4.x * xv);
        S[i].y = fmaf(g, S[i].y, b4.y * xv);
        S[i].z = fmaf(g, S[i].z, b4.z * xv);
        S[i].w = fmaf(g, S[i].w, b4.w * xv);
        r4[i] = fmaf(c4.w, S[i].w, fmaf(c4.z, S[i].z, fmaf(c4.y, S[i].y, c4.x * S[i].x)));
      }
      // the four columns' sums over the LPC lanes: two exchanges leave a lane with one column
      const bool odd = lane & 1, up = lane & 2;
      const float a0 = (odd ? r4[2] : r4[0]) + __shfl_xor(odd ? r4[0] : r4[2], 1, ZF_WAVE);
      const float a1 = (odd ? r4[3] : r4[1]) + __shfl_xor(odd ? r4[1] : r4[3], 1, ZF_WAVE);
      float r = (up ? a1 : a0) + __shfl_xor(up ? a0 : a1, 2, ZF_WAVE);
#pragma unroll
      for (int m = 4; m < LPC; m <<= 1) r += __shfl_xor(r, m, ZF_WAVE);
      const int mine = (wave * SS_NC + (odd ? 2 : 0) + (up ? 1 : 0)) * CPW + cl;
      if (cg < 4 && v0 + mine < p.dv)
        out[(size_t)(tc + t) * ((size_t)p.H * p.dv) + (size_t)hd * p.dv + v0 + mine] =
            fmaf(skip, xs[t * VBMAX + mine], r);
    }
  }
#pragma unroll
  for (int i = 0; i < SS_NC; ++i)
    if (t0 < t1 && live && v0 + col[i] < p.dv)
      *(float4*)(st + (size_t)(v0 + col[i]) * p.NP + 4 * cg) = S[i];
}

static bool ss_sizes(const StateSpace& p, long long slot_stride) {
  return p.H > 0 && p.G > 0 && p.H % p.G == 0 && p.N > 0 && p.dv > 0 && p.NP <= 256 &&
         slot_stride >= (long long)p.H * p.dv * p.NP && slot_stride % 4 == 0;
}

// seqs: the step's sequences to run (indices into q_start and state_slots), n_seqs of them; null:
// 0 .. n_seqs - 1.  steps null (bfloat16, every sequence one token): h [T, K] and w [H, K] instead.
extern "C" int zf_state_space_walk(const void* x, long long x_stride, const void* b, const void* c,
                                   long long bc_stride, int dtype, const float* steps,
                                   const float* a_log, const float* bias, const float* skip,
                                   float* state, long long slot_stride, const int* state_slots,
                                   const int* q_start, const int* seqs, float* out, int n_seqs,
                                   int H, int G, int N, int dv, const void* h, const void* w, int K,
                                   hipStream_t stream) {
  if (n_seqs <= 0) return 0;
  const bool own = steps == nullptr;
  const StateSpace p = {steps, a_log, bias, skip, H, G, N, dv, (N + 3) / 4 * 4,
                        own ? (const bf16_t*)h : nullptr, own ? (const bf16_t*)w : nullptr, K};
  if (!ss_sizes(p, slot_stride)) return -2;
  if (own && (dtype != ZF_BF16 || h == nullptr || w == nullptr || K % 8 != 0 || K <= 0 ||
              (uintptr_t)h % 16 != 0 || (uintptr_t)w % 16 != 0))
    return -2;
  int lpc = 4;
  while (4 * lpc < p.NP) lpc *= 2;
  const int per_wave = SS_NC * (ZF_WAVE / lpc);
  int waves = (dv + per_wave - 1) / per_wave;
  if (waves > 4) waves = 4;
  const dim3 grid(n_seqs, H, (dv + waves * per_wave - 1) / (waves * per_wave)), block(waves * ZF_WAVE);
#define SS_WALK(TT, L)                                                                           \
  hipLaunchKernelGGL((state_space_walk_kernel<TT, L>), grid, block, 0, stream, (const TT*)x,     \
                     x_stride, (const TT*)b, (const TT*)c, bc_stride, p, state, slot_stride,     \
                     state_slots, q_start, seqs, out)
#define SS_WALK_ANY(TT)                                                                          \
  if (lpc == 4) SS_WALK(TT, 4);                                                                  \
  else if (lpc == 8) SS_WALK(TT, 8);                                                             \
  else if (lpc == 16) SS_WALK(TT, 16);                                                           \
  else if (lpc == 32) SS_WALK(TT, 32);                                                           \
  else SS_WALK(TT, 64)
  if (dtype == ZF_F32) { SS_WALK_ANY(float); } else { SS_WALK_ANY(bf16_t); }
  ZF_CHECK_LAUNCH();
}

// ---------------------------------------------------------------- chunks side by side
#define SS_HEADS_MAX 4           // heads of one group a workgroup takes one after the other

struct StateSpaceChunks {
  const int* chunks;           // [n_chunks][4]: sequence, first token, tokens, -
  const int* firsts;           // [n_long][3]: sequence, first chunk, chunks
  float2* decays;              // [n_chunks][H][FC_C]: (L_t log2 e, dt_t); L stays where tokens end
  float* states;               // [n_chunks][H][dv][NP]
  int wide;                    // rows' groups of 8 lie at multiples of 16 bytes, N and dv % 8 == 0
  int heads;                   // heads a workgroup takes (a divisor of H / G)
};

// the elements c .. c + 7 of a row (zeros from `width` on), as they lie
__device__ __forceinline__ fc_u32x4_t ss_load8(const bf16_t* x, int c, int width, bool wide) {
  fc_u32x4_t v = {0u, 0u, 0u, 0u};
  if (wide) {
    if (c < width) v = *(const fc_u32x4_t*)(x + c);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const uint32_t a = c + 2 * i < width ? x[c + 2 * i] : 0;
      const uint32_t b = c + 2 * i + 1 < width ? x[c + 2 * i + 1] : 0;
      v[i] = a | (b << 16);
    }
  }
  return v;
}
__device__ __forceinline__ uint32_t ss_half(const fc_u32x4_t& v, int i) {
  return i & 1 ? v[i / 2] >> 16 : v[i / 2] & 0xffffu;
}

// a chunk's rows, transposed: [width columns][FC_C tokens]; x: the first row's first column wanted
template <int ROWS>
__device__ __forceinline__ void ss_stage_transposed(uint32_t* vt, const bf16_t* x, long long stride,
                                                    int n, int width, bool wide) {
  for (int task = threadIdx.x; task < (FC_C / 2) * (ROWS / 8); task += blockDim.x) {
    const int g = task % (ROWS / 8), tp = task / (ROWS / 8);
    fc_u32x4_t a = {0u, 0u, 0u, 0u}, b = {0u, 0u, 0u, 0u};
    const bf16_t* row = x + (size_t)(2 * tp) * stride;
    if (2 * tp < n) a = ss_load8(row, 8 * g, width, wide);
    if (2 * tp + 1 < n) b = ss_load8(row + stride, 8 * g, width, wide);
#pragma unroll
    for (int i = 0; i < 8; ++i) vt[fc_tr(8 * g + i, tp)] = ss_half(a, i) | (ss_half(b, i) << 16);
  }
}

// (1) a chunk's own sum over its tokens, sum_j exp(L_n - L_j) dt_j B_j x_j^T, to states[chunk], and
// the chunk's decays.  grid (chunk, block of heads, block of VB value columns), 4 waves; B lies
// transposed in LDS for all the heads; tiles of 32 columns x 32 channels are dealt over the waves.
template <int KD, int VB>
__global__ __launch_bounds__(256) void state_space_sums_kernel(
    const bf16_t* __restrict__ xr, long long x_stride, const bf16_t* __restrict__ br,
    long long bc_stride, StateSpace p, StateSpaceChunks a) {
  constexpr int TILES = (KD / 32) * (VB / 32), NT = (TILES + 3) / 4;
  __shared__ __attribute__((aligned(16))) uint32_t bt[KD * FC_C / 2];
  __shared__ __attribute__((aligned(16))) uint32_t xh[VB * FC_C / 2], xl[VB * FC_C / 2];
  __shared__ float Ls[SS_HEADS_MAX][FC_C], dts[SS_HEADS_MAX][FC_C];
  const int v0 = blockIdx.z * VB, first = blockIdx.y * a.heads;
  const int grp = first / (p.H / p.G);
  const int t0 = a.chunks[4 * blockIdx.x + 1], n = a.chunks[4 * blockIdx.x + 2];
  const int wave = threadIdx.x / 64, lane = threadIdx.x % 64, c = lane % 32, hl = lane / 32;
  // decays: a wave a head and half a chunk, summed over the lanes
  for (int u = wave; u < 2 * a.heads; u += 4) {
    const int h = u / 2, t = (u % 2) * 64 + lane;
    float dt = 0.f, L = 0.f;
    if (t < n) {
      dt = ss_softplus(p.steps[(size_t)(t0 + t) * p.H + first + h] + p.bias[first + h]);
      // (a token that keeps less than 2^-64 keeps nothing: the sums stay small numbers)
      L = fmaxf(-expf(p.a_log[first + h]) * dt * 1.4426950408889634f, -64.f);
    }
#pragma unroll
    for (int m = 1; m < 64; m <<= 1) {
      const float o = __shfl_up(L, m, ZF_WAVE);
      if (lane >= m) L += o;
    }
    Ls[h][t] = L;
    dts[h][t] = dt;
  }
  ss_stage_transposed<KD>(bt, br + (size_t)t0 * bc_stride + (size_t)grp * p.N, bc_stride, n, p.N,
                          a.wide);
  __syncthreads();
  for (int u = threadIdx.x; u < a.heads * FC_C / 2; u += 256) {
    const int h = u / (FC_C / 2), t = FC_C / 2 + u % (FC_C / 2);
    Ls[h][t] += Ls[h][FC_C / 2 - 1];
  }
  __syncthreads();
  if (blockIdx.z == 0)
    for (int u = threadIdx.x; u < a.heads * FC_C; u += 256) {
      const int h = u / FC_C, t = u % FC_C;
      a.decays[((size_t)blockIdx.x * p.H + first + h) * FC_C + t] = make_float2(Ls[h][t], dts[h][t]);
    }
  for (int h = 0; h < a.heads; ++h) {
    const int hd = first + h;
    const float total = Ls[h][FC_C - 1];
    const bf16_t* xp = xr + (size_t)t0 * x_stride + (size_t)hd * p.dv + v0;
    for (int task = threadIdx.x; task < (FC_C / 2) * (VB / 8); task += 256) {
      const int g = task % (VB / 8), tp = task / (VB / 8);
      fc_u32x4_t u = {0u, 0u, 0u, 0u}, v = {0u, 0u, 0u, 0u};
      const bf16_t* row = xp + (size_t)(2 * tp) * x_stride;
      if (2 * tp < n) u = ss_load8(row, 8 * g, p.dv - v0, a.wide);
      if (2 * tp + 1 < n) v = ss_load8(row + x_stride, 8 * g, p.dv - v0, a.wide);
      const float w0 = __builtin_amdgcn_exp2f(total - Ls[h][2 * tp]) * dts[h][2 * tp];
      const float w1 = __builtin_amdgcn_exp2f(total - Ls[h][2 * tp + 1]) * dts[h][2 * tp + 1];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        uint32_t lo;
        const int at = fc_tr(8 * g + i, tp);
        xh[at] = fc_pack(__uint_as_float(ss_half(u, i) << 16) * w0,
                         __uint_as_float(ss_half(v, i) << 16) * w1, lo);
        xl[at] = lo;
      }
    }
    __syncthreads();
    float* st = a.states + ((size_t)blockIdx.x * p.H + hd) * ((size_t)p.dv * p.NP);
#pragma unroll
    for (int u = 0; u < NT; ++u) {
      const int tile = wave + u * 4;
      if (tile >= TILES) break;
      const int vb = (tile / (KD / 32)) * 32, kb = (tile % (KD / 32)) * 32;
      if (v0 + vb >= p.dv || kb >= p.NP) continue;
      fc_f32x16_t acc;
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[r] = 0.f;
#pragma unroll
      for (int i = 0; i < FC_C / 16; ++i) {
        const fc_u32x4_t bv = *(const fc_u32x4_t*)(bt + fc_tr(kb + c, 8 * i + 4 * hl));
        const fc_u32x4_t ah = *(const fc_u32x4_t*)(xh + fc_tr(vb + c, 8 * i + 4 * hl));
        const fc_u32x4_t al = *(const fc_u32x4_t*)(xl + fc_tr(vb + c, 8 * i + 4 * hl));
        acc = fc_mfma(ah, bv, acc);
        acc = fc_mfma(al, bv, acc);
      }
      // acc[r]: value column vb + 8 (r / 4) + 4 hl + r % 4, channel kb + c
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int col = v0 + vb + 8 * (r / 4) + 4 * hl + r % 4;
        if (col < p.dv && kb + c < p.NP) st[(size_t)col * p.NP + kb + c] = acc[r];
      }
    }
    __syncthreads();                                 // the weighted rows are read
  }
}

// (2) the states at the chunks' starts: states[chunk] becomes the state before the chunk, the one
// behind the last goes to the request's slot.  A thread walks 4 neighbouring entries; grid
// (blocks of entries, long sequence).
#define SS_AHEAD 8
__global__ __launch_bounds__(256) void state_space_states_kernel(
    StateSpace p, StateSpaceChunks a, float* __restrict__ state, long long slot_stride,
    const int* __restrict__ state_slots) {
  const long long size = (long long)p.H * p.dv * p.NP;
  const long long e = ((long long)blockIdx.x * blockDim.x + threadIdx.x) * 4;
  if (e >= size) return;
  const int s = a.firsts[3 * blockIdx.y], first = a.firsts[3 * blockIdx.y + 1],
            count = a.firsts[3 * blockIdx.y + 2];
  const int hd = (int)(e / ((long long)p.dv * p.NP));
  float* st = state + (size_t)state_slots[s] * slot_stride + e;
  float* at = a.states + (size_t)first * size + e;
  const float2* dec = a.decays + ((size_t)first * p.H + hd) * FC_C + FC_C - 1;
  float4 S = *(const float4*)st;
  for (int n0 = 0; n0 < count; n0 += SS_AHEAD) {
    float4 own[SS_AHEAD];
    float g[SS_AHEAD];
#pragma unroll
    for (int u = 0; u < SS_AHEAD; ++u)
      if (n0 + u < count) {
        own[u] = *(const float4*)(at + (size_t)(n0 + u) * size);
        g[u] = __builtin_amdgcn_exp2f(dec[(size_t)(n0 + u) * p.H * FC_C].x);
      }
#pragma unroll
    for (int u = 0; u < SS_AHEAD; ++u)
      if (n0 + u < count) {
        *(float4*)(at + (size_t)(n0 + u) * size) = S;
        S = float4{fmaf(g[u], S.x, own[u].x), fmaf(g[u], S.y, own[u].y), fmaf(g[u], S.z, own[u].z),
                   fmaf(g[u], S.w, own[u].w)};
      }
  }
  *(float4*)st = S;
}

// (3) a chunk's outputs.  grid (chunk, block of heads, block of VB value columns), 4 waves; a wave
// takes 32 queries.  B's rows lie in LDS first, for the scores C . B, which are the same for every
// head of the group and stay in registers (computed as B C^T, so that a lane's 16 numbers of a
// block of 32 keys belong to one query and go from registers into the second product).  Then head
// by head the state (S^T, rows of KD channels) takes their place, beside it the head's x
// transposed.
template <int KD, int VB>
__global__ __launch_bounds__(256, 2) void state_space_outputs_kernel(
    const bf16_t* __restrict__ xr, long long x_stride, const bf16_t* __restrict__ br,
    const bf16_t* __restrict__ cr, long long bc_stride, StateSpace p, StateSpaceChunks a,
    float* __restrict__ out) {
  constexpr int ROWS = 2 * VB > FC_C ? 2 * VB : FC_C;
  __shared__ __attribute__((aligned(16))) bf16_t rows[ROWS * KD];
  __shared__ __attribute__((aligned(16))) uint32_t vt[VB * FC_C / 2];
  __shared__ float2 dec[FC_C];
  const int v0 = blockIdx.z * VB, first = blockIdx.y * a.heads;
  const int grp = first / (p.H / p.G);
  const int t0 = a.chunks[4 * blockIdx.x + 1], n = a.chunks[4 * blockIdx.x + 2];
  const int wave = threadIdx.x / 64, lane = threadIdx.x % 64, c = lane % 32, hl = lane / 32;
  const int qb = wave;
  const int i_q = 32 * qb + c;                        // this lane's query
  const bool q_ok = i_q < n;
  // the wave's queries, channels 16 i + 8 hl .. of every i
  fc_u32x4_t q[KD / 16];
  {
    const bf16_t* row = cr + (size_t)(t0 + (q_ok ? i_q : 0)) * bc_stride + (size_t)grp * p.N;
#pragma unroll
    for (int i = 0; i < KD / 16; ++i) {
      q[i] = ss_load8(row, 16 * i + 8 * hl, p.N, a.wide);
      if (!q_ok) q[i] = fc_u32x4_t{0u, 0u, 0u, 0u};
    }
  }
  for (int task = threadIdx.x; task < FC_C * (KD / 8); task += 256) {
    const int g = task % (KD / 8), t = task / (KD / 8);
    fc_u32x4_t v = {0u, 0u, 0u, 0u};
    if (t < n) v = ss_load8(br + (size_t)(t0 + t) * bc_stride + (size_t)grp * p.N, 8 * g, p.N, a.wide);
    *(fc_u32x4_t*)(rows + fc_row<KD>(t, g)) = v;
  }
  __syncthreads();
  fc_f32x16_t sc[FC_C / 32];
#pragma unroll
  for (int kb = 0; kb < FC_C / 32; ++kb) {
#pragma unroll
    for (int r = 0; r < 16; ++r) sc[kb][r] = 0.f;
    if (kb <= qb) {
#pragma unroll
      for (int i = 0; i < KD / 16; ++i) {
        const fc_u32x4_t k = *(const fc_u32x4_t*)(rows + fc_row<KD>(32 * kb + c, 2 * i + hl));
        sc[kb] = fc_mfma(k, q[i], sc[kb]);
      }
      // sc[kb][r]: key 32 kb + 8 (r / 4) + 4 hl + r % 4, this lane's query
      if (kb == qb) {
#pragma unroll
        for (int r = 0; r < 16; ++r)
          if (8 * (r / 4) + 4 * hl + r % 4 > c) sc[kb][r] = 0.f;
      }
    }
  }
  for (int h = 0; h < a.heads; ++h) {
    const int hd = first + h;
    __syncthreads();                                 // B's rows, or the head before, are read
    const size_t at_state = ((size_t)blockIdx.x * p.H + hd) * ((size_t)p.dv * p.NP);
    for (int task = threadIdx.x; task < VB * (KD / 8); task += 256) {
      const int g = task % (KD / 8), r = task / (KD / 8);
      float x[8];
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        float4 f = float4{0.f, 0.f, 0.f, 0.f};
        if (v0 + r < p.dv && 8 * g + 4 * u < p.NP)
          f = *(const float4*)(a.states + at_state + (size_t)(v0 + r) * p.NP + 8 * g + 4 * u);
        x[4 * u] = f.x; x[4 * u + 1] = f.y; x[4 * u + 2] = f.z; x[4 * u + 3] = f.w;
      }
      fc_u32x4_t hi, lo;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        uint32_t l;
        hi[i] = fc_pack(x[2 * i], x[2 * i + 1], l);
        lo[i] = l;
      }
      *(fc_u32x4_t*)(rows + fc_row<KD>(r, g)) = hi;
      *(fc_u32x4_t*)(rows + fc_row<KD>(VB + r, g)) = lo;
    }
    ss_stage_transposed<VB>(vt, xr + (size_t)t0 * x_stride + (size_t)hd * p.dv + v0, x_stride, n,
                            p.dv - v0, a.wide);
    if (threadIdx.x < FC_C)
      dec[threadIdx.x] = a.decays[((size_t)blockIdx.x * p.H + hd) * FC_C + threadIdx.x];
    __syncthreads();
    if (32 * qb >= n) continue;                      // (a whole wave; it meets the barriers above)
    const float Lq = dec[i_q].x;
    const float skip = p.skip[hd];
    fc_f32x16_t acc[VB / 32];
#pragma unroll
    for (int j = 0; j < VB / 32; ++j) {
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[j][r] = 0.f;
#pragma unroll
      for (int i = 0; i < KD / 16; ++i) {
        const fc_u32x4_t sh = *(const fc_u32x4_t*)(rows + fc_row<KD>(32 * j + c, 2 * i + hl));
        const fc_u32x4_t sl = *(const fc_u32x4_t*)(rows + fc_row<KD>(VB + 32 * j + c, 2 * i + hl));
        acc[j] = fc_mfma(sh, q[i], acc[j]);
        acc[j] = fc_mfma(sl, q[i], acc[j]);
      }
      const float g = __builtin_amdgcn_exp2f(Lq);
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[j][r] *= g;
    }
#pragma unroll
    for (int kb = 0; kb < FC_C / 32; ++kb) {
      if (kb > qb) break;
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        // the registers 8 t .. 8 t + 7: keys 16 t + {0..3, 8..11} + 4 hl, and x^T in that order
        float w[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int r = 8 * t + e;
          const int j = 32 * kb + 8 * (r / 4) + 4 * hl + r % 4;
          const float2 d = dec[j];
          w[e] = sc[kb][r] * (__builtin_amdgcn_exp2f(fminf(Lq - d.x, 0.f)) * d.y);
        }
        fc_u32x4_t ph, pl;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          uint32_t lo;
          ph[e] = fc_pack(w[2 * e], w[2 * e + 1], lo);
          pl[e] = lo;
        }
#pragma unroll
        for (int j = 0; j < VB / 32; ++j) {
          const uint2 a0 = *(const uint2*)(vt + fc_tr(32 * j + c, 16 * kb + 8 * t + 2 * hl));
          const uint2 a1 = *(const uint2*)(vt + fc_tr(32 * j + c, 16 * kb + 8 * t + 4 + 2 * hl));
          const fc_u32x4_t av = {a0.x, a0.y, a1.x, a1.y};
          acc[j] = fc_mfma(av, ph, acc[j]);
          acc[j] = fc_mfma(av, pl, acc[j]);
        }
      }
    }
    if (!q_ok) continue;
    const bf16_t* xq = xr + (size_t)(t0 + i_q) * x_stride + (size_t)hd * p.dv;
    float* o = out + (size_t)(t0 + i_q) * ((size_t)p.H * p.dv) + (size_t)hd * p.dv;
#pragma unroll
    for (int j = 0; j < VB / 32; ++j)
#pragma unroll
      for (int r4 = 0; r4 < 4; ++r4) {
        const int col = v0 + 32 * j + 8 * r4 + 4 * hl;
        if (a.wide) {
          if (col < p.dv) {
            const uint2 x = *(const uint2*)(xq + col);
            *(float4*)(o + col) = float4{fmaf(skip, __uint_as_float(x.x << 16), acc[j][4 * r4]),
                                         fmaf(skip, __uint_as_float(x.x & 0xffff0000u), acc[j][4 * r4 + 1]),
                                         fmaf(skip, __uint_as_float(x.y << 16), acc[j][4 * r4 + 2]),
                                         fmaf(skip, __uint_as_float(x.y & 0xffff0000u), acc[j][4 * r4 + 3])};
          }
        } else {
#pragma unroll
          for (int x = 0; x < 4; ++x)
            if (col + x < p.dv) o[col + x] = fmaf(skip, bf16_to_float(xq[col + x]), acc[j][4 * r4 + x]);
        }
      }
  }
}

// chunks [n_chunks][4] and firsts [n_long][3] (device, int32) list the chunks of the step's long
// sequences: chunk c of sequence chunks[c][0] holds the tokens chunks[c][1] .. + chunks[c][2] - 1
// (of the step), a sequence's chunks lie in order, all of FC_C tokens but its last; firsts: the
// sequence, its first chunk, how many.  Scratch: states float32 [n_chunks, H dv NP], decays float32
// [n_chunks, H, FC_C, 2].  heads: how many heads a workgroup takes, a divisor of H / G up to 4.
extern "C" int zf_state_space_chunks(const void* x, long long x_stride, const void* b, const void* c,
                                     long long bc_stride, const float* steps, const float* a_log,
                                     const float* bias, const float* skip, float* state,
                                     long long slot_stride, const int* state_slots,
                                     const int* chunks, int n_chunks, const int* firsts, int n_long,
                                     float* states, float* decays, float* out, int H, int G, int N,
                                     int dv, int heads, hipStream_t stream) {
  if (n_chunks <= 0 || n_long <= 0) return 0;
  const StateSpace p = {steps, a_log, bias, skip, H, G, N, dv, (N + 3) / 4 * 4, nullptr, nullptr, 0};
  if (!ss_sizes(p, slot_stride) || states == nullptr || decays == nullptr || heads < 1 ||
      heads > SS_HEADS_MAX || (H / G) % heads != 0)
    return -2;
  StateSpaceChunks a;
  a.chunks = chunks; a.firsts = firsts; a.decays = (float2*)decays; a.states = states;
  a.heads = heads;
  a.wide = N % 8 == 0 && dv % 8 == 0 && x_stride % 8 == 0 && bc_stride % 8 == 0 &&
           (uintptr_t)x % 16 == 0 && (uintptr_t)b % 16 == 0 && (uintptr_t)c % 16 == 0;
  const bf16_t *xp = (const bf16_t*)x, *bp = (const bf16_t*)b, *cp = (const bf16_t*)c;
  const long long quads = (long long)H * dv * p.NP / 4;
#define SS_RUN(KD, VB)                                                                            \
  {                                                                                              \
    const dim3 grid(n_chunks, H / heads, (dv + VB - 1) / VB);                                    \
    hipLaunchKernelGGL((state_space_sums_kernel<KD, VB>), grid, dim3(256), 0, stream, xp,        \
                       x_stride, bp, bc_stride, p, a);                                           \
    hipLaunchKernelGGL(state_space_states_kernel, dim3((unsigned)((quads + 255) / 256), n_long), \
                       dim3(256), 0, stream, p, a, state, slot_stride, state_slots);             \
    hipLaunchKernelGGL((state_space_outputs_kernel<KD, VB>), grid, dim3(256), 0, stream, xp,     \
                       x_stride, bp, cp, bc_stride, p, a, out);                                  \
  }
#define SS_RUN_VB(KD)                                                                            \
  if (dv <= 32) SS_RUN(KD, 32)                                                                   \
  else SS_RUN(KD, 64)
  if (N <= 32) { SS_RUN_VB(32) }
  else if (N <= 64) { SS_RUN_VB(64) }
  else if (N <= 128) { SS_RUN_VB(128) }
  else SS_RUN(256, 32)
  ZF_CHECK_LAUNCH();
}
