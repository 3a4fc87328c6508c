// Linear attention with one fixed decay a head: a matrix S [d, dv] a head in 32-bit,
//
//   S_t = g S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t          (g in [0, 1], one number a head)
//
// with what stands between a projection's rows and the recurrence done on the way in, a head's
// elements as floats: silu of q, k and v (or not), a
// rotation of q's and k's leading elements by the token's position (pairs (i, i + dims / 2),
// cosines and sines from a table a token), a factor on k.
//
//  * rotation_table      cosine and sine of position * frequency, a row a token
//  * fixed_decay_walk    token by token, every size, both storage types, all 32-bit: single
//                        tokens, short portions and the whole 32-bit path
//  * fixed_decay_chunks  bfloat16 rows, portions in chunks of 128 tokens side by side.  With S the
//                        state before a chunk, i and j tokens of it counted from 0:
//                          o_i = g^(i+1) S^T q_i + sum_j<=i g^(i-j) (q_i . k_j) v_j
//                          S  <- g^n S + sum_j g^(n-1-j) k_j v_j^T
//                        which are matrix products: (1) every chunk's own sum, (2) the states at
//                        the chunks' starts one after the other, (3) every chunk's outputs.  The
//                        products run in bfloat16 MFMAs with 32-bit sums; an operand that is a
//                        32-bit number (q and k behind the rotation, the weighted k, the weights
//                        g^(i-j) q . k, the state) enters as the sum of two bfloat16 numbers, its
//                        rounding and the rounding of what that leaves (2^-16 relative).
//
// A request's state is laid out [head][value column][channels padded to 4].
#include "zf_chunks.h"

// ---------------------------------------------------------------- the rotation's table
// grid (blocks of pairs, tokens): out[t][j] = (cos, sin) of positions[t] * freq[j], times mag
__global__ void rotation_table_kernel(const int* __restrict__ positions,
                                      const float* __restrict__ freq, float mag,
                                      float2* __restrict__ out, int half) {
  const int j = blockIdx.x * blockDim.x + threadIdx.x;
  if (j >= half) return;
  float sn, cs;
  sincosf((float)positions[blockIdx.y] * freq[j], &sn, &cs);
  out[(size_t)blockIdx.y * half + j] = make_float2(cs * mag, sn * mag);
}

extern "C" int zf_rotation_table(const int* positions, const float* freq, float mag, float* out,
                                 int T, int half, hipStream_t stream) {
  if (T <= 0 || half <= 0) return 0;
  hipLaunchKernelGGL(rotation_table_kernel, dim3((half + 63) / 64, T), dim3(64), 0, stream,
                     positions, freq, mag, (float2*)out, half);
  ZF_CHECK_LAUNCH();
}

// ---------------------------------------------------------------- rows on their way in
struct FixedDecayRows {
  long long q_stride, k_stride, v_stride;      // elements from one row to the next
  const float2* table;                         // [T][half]; null: no rotation
  int half;
  int silu;                                    // q, k and v pass silu first
  float k_scale;
};

template <typename T>
__device__ __forceinline__ float fd_value(const T* x, int c, int silu) {
  const float v = load_as_float<T>(x + c);
  return silu ? v / (1.0f + expf(-v)) : v;
}
// element c of a head's row x, as it enters the recurrence
template <typename T>
__device__ __forceinline__ float fd_element(const T* x, int c, const float2* tab, int half, int silu) {
  const float a = fd_value<T>(x, c, silu);
  if (tab == nullptr || c >= 2 * half) return a;
  const bool first = c < half;
  const float b = fd_value<T>(x, first ? c + half : c - half, silu);
  const float2 cs = tab[first ? c : c - half];
  return first ? a * cs.x - b * cs.y : a * cs.x + b * cs.y;
}

// ---------------------------------------------------------------- token by token
// grid (sequence, head, block of value columns); a wave's lanes hold LPC lanes of 4 channels for
// each of 64 / LPC value columns side by side, FD_NC such groups of columns one behind the other.
// Eight tokens' rows at a time lie in LDS as floats.  A column's partial outputs are added over
// its lanes in an order that depends on LPC alone.
#define FD_NC 4
#define FD_TC 8

template <typename T, int LPC>
__global__ __launch_bounds__(256) void fixed_decay_walk_kernel(
    const T* __restrict__ q, const T* __restrict__ k, const T* __restrict__ v, FixedDecayRows rows,
    const float* __restrict__ decay, float* __restrict__ state, long long slot_stride,
    const int* __restrict__ state_slots, const int* __restrict__ q_start,
    const int* __restrict__ seqs, float* __restrict__ out, int H, int d, int dv, int DP) {
  constexpr int CPW = ZF_WAVE / LPC;                 // columns side by side in a wave
  constexpr int KW = 4 * LPC;
  constexpr int VBMAX = 4 * FD_NC * CPW;
  __shared__ __attribute__((aligned(16))) float qs[FD_TC * KW], ks[FD_TC * KW];
  __shared__ float vs[FD_TC * VBMAX];
  const int s = seqs != nullptr ? seqs[blockIdx.x] : blockIdx.x;
  const int hd = blockIdx.y;
  const int t0 = q_start[s], t1 = q_start[s + 1];
  const int tid = threadIdx.x, wave = tid / ZF_WAVE, lane = tid % ZF_WAVE;
  const int VB = (blockDim.x / ZF_WAVE) * FD_NC * CPW;
  const int v0 = blockIdx.z * VB;
  const int cg = lane % LPC, cl = lane / LPC;
  const bool live = 4 * cg < DP;
  float* st = state + (size_t)state_slots[s] * slot_stride + (size_t)hd * dv * DP;
  float4 S[FD_NC];
  int col[FD_NC];
#pragma unroll
  for (int i = 0; i < FD_NC; ++i) {
    col[i] = (wave * FD_NC + i) * CPW + cl;          // within the block
    S[i] = float4{0.f, 0.f, 0.f, 0.f};
    if (live && v0 + col[i] < dv) S[i] = *(const float4*)(st + (size_t)(v0 + col[i]) * DP + 4 * cg);
  }
  const float g = decay[hd];
  for (int tc = t0; tc < t1; tc += FD_TC) {
    const int n = min(FD_TC, t1 - tc);
    __syncthreads();                                 // the rows before are done with
    for (int i = tid; i < n * KW; i += blockDim.x) {
      const int t = i / KW, c = i % KW;
      float qv = 0.f, kv = 0.f;
      if (c < d) {
        const size_t row = (size_t)(tc + t);
        const float2* tab = rows.table != nullptr ? rows.table + row * rows.half : nullptr;
        qv = fd_element<T>(q + row * rows.q_stride + (size_t)hd * d, c, tab, rows.half, rows.silu);
        kv = fd_element<T>(k + row * rows.k_stride + (size_t)hd * d, c, tab, rows.half, rows.silu)
             * rows.k_scale;
      }
      qs[i] = qv;
      ks[i] = kv;
    }
    for (int i = tid; i < n * VB; i += blockDim.x) {
      const int t = i / VB, x = i % VB;
      vs[t * VBMAX + x] = v0 + x < dv
          ? fd_value<T>(v + (size_t)(tc + t) * rows.v_stride + (size_t)hd * dv, v0 + x, rows.silu) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < n; ++t) {
      const float4 q4 = *(const float4*)(qs + t * KW + 4 * cg);
      const float4 k4 = *(const float4*)(ks + t * KW + 4 * cg);
      float p[FD_NC];
#pragma unroll
      for (int i = 0; i < FD_NC; ++i) {
        const float vv = vs[t * VBMAX + col[i]];
        S[i].x = fmaf(g, S[i].x, k4.x * vv);
        S[i].y = fmaf(g, S[i].y, k4.y * vv);
        S[i].z = fmaf(g, S[i].z, k4.z * vv);
        S[i].w = fmaf(g, S[i].w, k4.w * vv);
        p[i] = fmaf(q4.w, S[i].w, fmaf(q4.z, S[i].z, fmaf(q4.y, S[i].y, q4.x * S[i].x)));
      }
      // the four columns' sums over the LPC lanes: two exchanges leave a lane with one column
      const bool odd = lane & 1, up = lane & 2;
      const float a0 = (odd ? p[2] : p[0]) + __shfl_xor(odd ? p[0] : p[2], 1, ZF_WAVE);
      const float a1 = (odd ? p[3] : p[1]) + __shfl_xor(odd ? p[1] : p[3], 1, ZF_WAVE);
      float r = (up ? a1 : a0) + __shfl_xor(up ? a0 : a1, 2, ZF_WAVE);
#pragma unroll
      for (int m = 4; m < LPC; m <<= 1) r += __shfl_xor(r, m, ZF_WAVE);
      const int mine = (wave * FD_NC + (odd ? 2 : 0) + (up ? 1 : 0)) * CPW + cl;
      if (cg < 4 && v0 + mine < dv)
        out[(size_t)(tc + t) * ((size_t)H * dv) + (size_t)hd * dv + v0 + mine] = r;
    }
  }
#pragma unroll
  for (int i = 0; i < FD_NC; ++i)
    if (t0 < t1 && live && v0 + col[i] < dv)
      *(float4*)(st + (size_t)(v0 + col[i]) * DP + 4 * cg) = S[i];
}

// seqs: the step's sequences to run (indices into q_start and state_slots), n_seqs of them; null:
// 0 .. n_seqs - 1
extern "C" int zf_fixed_decay_walk(const void* q, long long q_stride, const void* k,
                                   long long k_stride, const void* v, long long v_stride, int dtype,
                                   const float* table, int half, int silu, float k_scale,
                                   const float* decay, float* state, long long slot_stride,
                                   const int* state_slots, const int* q_start, const int* seqs,
                                   float* out, int n_seqs, int H, int d, int dv,
                                   hipStream_t stream) {
  if (n_seqs <= 0) return 0;
  const int DP = (d + 3) / 4 * 4;
  if (H <= 0 || d <= 0 || dv <= 0 || DP > 256 || slot_stride < (long long)H * dv * DP ||
      slot_stride % 4 != 0 || 2 * half > d || (table != nullptr && half <= 0))
    return -2;
  FixedDecayRows rows;
  rows.q_stride = q_stride; rows.k_stride = k_stride; rows.v_stride = v_stride;
  rows.table = (const float2*)table; rows.half = half; rows.silu = silu; rows.k_scale = k_scale;
  int lpc = 4;
  while (4 * lpc < DP) lpc *= 2;
  const int per_wave = FD_NC * (ZF_WAVE / lpc);
  int waves = (dv + per_wave - 1) / per_wave;
  if (waves > 4) waves = 4;
  const dim3 grid(n_seqs, H, (dv + waves * per_wave - 1) / (waves * per_wave)), block(waves * ZF_WAVE);
#define FD_WALK(TT, L)                                                                           \
  hipLaunchKernelGGL((fixed_decay_walk_kernel<TT, L>), grid, block, 0, stream, (const TT*)q,     \
                     (const TT*)k, (const TT*)v, rows, decay, state, slot_stride, state_slots,   \
                     q_start, seqs, out, H, d, dv, DP)
#define FD_WALK_ANY(TT)                                                                          \
  if (lpc == 4) FD_WALK(TT, 4);                                                                  \
  else if (lpc == 8) FD_WALK(TT, 8);                                                             \
  else if (lpc == 16) FD_WALK(TT, 16);                                                           \
  else if (lpc == 32) FD_WALK(TT, 32);                                                           \
  else FD_WALK(TT, 64)
  if (dtype == ZF_F32) { FD_WALK_ANY(float); } else { FD_WALK_ANY(bf16_t); }
  ZF_CHECK_LAUNCH();
}

// ---------------------------------------------------------------- chunks side by side
__device__ __forceinline__ float fc_silu(float v) {
  return v * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * v));
}

// the elements c .. c + 7 of a head's row as floats, activated (0 from `width` on); `wide`: the
// row's groups of 8 lie at multiples of 16 bytes and width is a multiple of 8
__device__ __forceinline__ void fc_raw8(const bf16_t* x, int c, int width, int silu, bool wide,
                                        float (&o)[8]) {
  if (wide) {
    uint4 r = make_uint4(0u, 0u, 0u, 0u);
    if (c < width) r = *(const uint4*)(x + c);
    const uint32_t w[4] = {r.x, r.y, r.z, r.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      o[2 * i] = __uint_as_float(w[i] << 16);
      o[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) o[i] = c + i < width ? bf16_to_float(x[c + i]) : 0.f;
  }
  if (silu)
#pragma unroll
    for (int i = 0; i < 8; ++i) o[i] = fc_silu(o[i]);           // (silu of 0 is 0)
}
// the same behind the rotation; `wide` rows turn whole groups (half a multiple of 8)
__device__ __forceinline__ void fc_turned8(const bf16_t* x, int c, int width, const float2* tab,
                                           int half, int silu, bool wide, float (&o)[8]) {
  fc_raw8(x, c, width, silu, wide, o);
  if (tab == nullptr || c >= 2 * half) return;
  if (wide) {
    const bool first = c < half;
    float b[8];
    fc_raw8(x, first ? c + half : c - half, width, silu, true, b);
    const float4* tp = (const float4*)(tab + (first ? c : c - half));
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float4 cs = tp[i];
      o[2 * i] = first ? o[2 * i] * cs.x - b[2 * i] * cs.y : o[2 * i] * cs.x + b[2 * i] * cs.y;
      o[2 * i + 1] = first ? o[2 * i + 1] * cs.z - b[2 * i + 1] * cs.w
                           : o[2 * i + 1] * cs.z + b[2 * i + 1] * cs.w;
    }
  } else {
    for (int i = 0; i < 8; ++i)
      if (c + i < 2 * half) o[i] = fd_element<bf16_t>(x, c + i, tab, half, silu);
  }
}

// the chunk's values, transposed: [VB value columns][FC_C tokens] as bfloat16
template <int VB>
__device__ __forceinline__ void fc_stage_values(uint32_t* vt, const bf16_t* v, long long v_stride,
                                                int hd, int dv, int v0, int t0, int n, int silu,
                                                bool wide) {
  for (int task = threadIdx.x; task < (FC_C / 2) * (VB / 8); task += blockDim.x) {
    const int g = task % (VB / 8), tp = task / (VB / 8);
    float a[8], b[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) a[i] = b[i] = 0.f;
    const bf16_t* x = v + (size_t)(t0 + 2 * tp) * v_stride + (size_t)hd * dv;
    if (2 * tp < n) fc_raw8(x, v0 + 8 * g, dv, silu, wide, a);
    if (2 * tp + 1 < n) fc_raw8(x + v_stride, v0 + 8 * g, dv, silu, wide, b);
#pragma unroll
    for (int i = 0; i < 8; ++i) vt[fc_tr(8 * g + i, tp)] = pack_bf16x2(a[i], b[i]);
  }
}

struct FixedDecayChunks {
  const int* chunks;           // [n_chunks][4]: sequence, first token, tokens, -
  const int* firsts;           // [n_long][3]: sequence, first chunk, chunks
  const float* log2g;          // [H]
  float* states;               // [n_chunks][H][dv][DP]
  int H, d, dv, DP, wide;
};

// (1) a chunk's own sum over its tokens, sum_j g^(n-1-j) k_j v_j^T, to states[chunk].
// grid (chunk, head, block of VB value columns), NW waves; tiles of 32 columns x 32 channels are
// dealt over the waves.
template <int KD, int VB, int NW>
__global__ __launch_bounds__(NW * 64) void fixed_decay_sums_kernel(
    const bf16_t* __restrict__ k, const bf16_t* __restrict__ v, FixedDecayRows rows,
    FixedDecayChunks a) {
  constexpr int TILES = (KD / 32) * (VB / 32), NT = (TILES + NW - 1) / NW;
  __shared__ __attribute__((aligned(16))) uint32_t kh[KD * FC_C / 2], kl[KD * FC_C / 2];
  __shared__ __attribute__((aligned(16))) uint32_t vt[VB * FC_C / 2];
  const int hd = blockIdx.y, v0 = blockIdx.z * VB;
  const int t0 = a.chunks[4 * blockIdx.x + 1], n = a.chunks[4 * blockIdx.x + 2];
  const int wave = threadIdx.x / 64, lane = threadIdx.x % 64, c = lane % 32, hl = lane / 32;
  const float lg = a.log2g[hd];
  for (int task = threadIdx.x; task < (FC_C / 2) * (KD / 8); task += NW * 64) {
    const int g = task % (KD / 8), tp = task / (KD / 8);
    float x[2][8];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int t = 2 * tp + u;
#pragma unroll
      for (int i = 0; i < 8; ++i) x[u][i] = 0.f;
      if (t < n) {
        const size_t row = (size_t)(t0 + t);
        const float2* tab = rows.table != nullptr ? rows.table + row * rows.half : nullptr;
        fc_turned8(k + row * rows.k_stride + (size_t)hd * a.d, 8 * g, a.d, tab, rows.half, rows.silu,
                   a.wide, x[u]);
        const float w = rows.k_scale * fc_pow(lg, n - 1 - t);
#pragma unroll
        for (int i = 0; i < 8; ++i) x[u][i] *= w;
      }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      uint32_t lo;
      const int at = fc_tr(8 * g + i, tp);
      kh[at] = fc_pack(x[0][i], x[1][i], lo);
      kl[at] = lo;
    }
  }
  fc_stage_values<VB>(vt, v, rows.v_stride, hd, a.dv, v0, t0, n, rows.silu, a.wide);
  __syncthreads();
  float* st = a.states + (size_t)blockIdx.x * ((size_t)a.H * a.dv * a.DP) + (size_t)hd * a.dv * a.DP;
#pragma unroll
  for (int u = 0; u < NT; ++u) {
    const int tile = wave + u * NW;
    if (tile >= TILES) break;
    const int vb = (tile / (KD / 32)) * 32, kb = (tile % (KD / 32)) * 32;
    if (v0 + vb >= a.dv || kb >= a.DP) continue;
    fc_f32x16_t acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.f;
#pragma unroll
    for (int i = 0; i < FC_C / 16; ++i) {
      const fc_u32x4_t av = *(const fc_u32x4_t*)(vt + fc_tr(vb + c, 8 * i + 4 * hl));
      const fc_u32x4_t bh = *(const fc_u32x4_t*)(kh + fc_tr(kb + c, 8 * i + 4 * hl));
      const fc_u32x4_t bl = *(const fc_u32x4_t*)(kl + fc_tr(kb + c, 8 * i + 4 * hl));
      acc = fc_mfma(av, bh, acc);
      acc = fc_mfma(av, bl, acc);
    }
    // acc[r]: value column vb + 8 (r / 4) + 4 hl + r % 4, channel kb + c
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int col = v0 + vb + 8 * (r / 4) + 4 * hl + r % 4;
      if (col < a.dv && kb + c < a.DP) st[(size_t)col * a.DP + kb + c] = acc[r];
    }
  }
}

// (2) the states at the chunks' starts: states[chunk] becomes the state before the chunk, the one
// behind the last goes to the request's slot.  A thread walks 4 neighbouring entries; grid
// (blocks of entries, long sequence).
#define FC_AHEAD 8
__global__ __launch_bounds__(256) void fixed_decay_states_kernel(
    FixedDecayChunks a, float* __restrict__ state, long long slot_stride,
    const int* __restrict__ state_slots) {
  const long long size = (long long)a.H * a.dv * a.DP;
  const long long e = ((long long)blockIdx.x * blockDim.x + threadIdx.x) * 4;
  if (e >= size) return;
  const int s = a.firsts[3 * blockIdx.y], first = a.firsts[3 * blockIdx.y + 1],
            count = a.firsts[3 * blockIdx.y + 2];
  const float lg = a.log2g[e / ((long long)a.dv * a.DP)];
  float* st = state + (size_t)state_slots[s] * slot_stride + e;
  float* at = a.states + (size_t)first * size + e;
  float4 S = *(const float4*)st;
  for (int n0 = 0; n0 < count; n0 += FC_AHEAD) {
    float4 own[FC_AHEAD];
#pragma unroll
    for (int u = 0; u < FC_AHEAD; ++u)
      if (n0 + u < count) own[u] = *(const float4*)(at + (size_t)(n0 + u) * size);
#pragma unroll
    for (int u = 0; u < FC_AHEAD; ++u)
      if (n0 + u < count) {
        *(float4*)(at + (size_t)(n0 + u) * size) = S;
        const float g = fc_pow(lg, a.chunks[4 * (first + n0 + u) + 2]);
        S = float4{fmaf(g, S.x, own[u].x), fmaf(g, S.y, own[u].y), fmaf(g, S.z, own[u].z),
                   fmaf(g, S.w, own[u].w)};
      }
  }
  *(float4*)st = S;
}

// (3) a chunk's outputs.  grid (chunk, head, block of VB value columns); 4 VH waves: wave w takes
// the 32 queries of block w % 4 and the value columns of part w / 4 (VB / VH of them).  The chunk's
// values lie transposed in LDS, beside them first the state (S^T, rows of KD channels) for
// g^(i+1) S^T q_i, then the chunk's keys (rows of KD channels) for the rest.  Scores are computed as K Q^T, so
// that a lane's 16 numbers belong to one query and go from registers into the second product.
template <int KD, int VB, int VH>
__global__ __launch_bounds__(VH * 256) void fixed_decay_outputs_kernel(
    const bf16_t* __restrict__ q, const bf16_t* __restrict__ k, const bf16_t* __restrict__ v,
    FixedDecayRows rows, FixedDecayChunks a, float* __restrict__ out) {
  constexpr int VW = VB / VH;                        // value columns of a wave
  constexpr int ROWS = VB > FC_C ? VB : FC_C;
  __shared__ __attribute__((aligned(16))) bf16_t xh[ROWS * KD], xl[ROWS * KD];
  __shared__ __attribute__((aligned(16))) uint32_t vt[VB * FC_C / 2];
  const int hd = blockIdx.y, v0 = blockIdx.z * VB;
  const int t0 = a.chunks[4 * blockIdx.x + 1], n = a.chunks[4 * blockIdx.x + 2];
  const int wave = threadIdx.x / 64, lane = threadIdx.x % 64, c = lane % 32, hl = lane / 32;
  const int part = wave / 4;
  const int qb = part & 1 ? 3 - wave % 4 : wave % 4;  // (the last block walks the most keys)
  const float lg = a.log2g[hd];
  const int i_q = 32 * qb + c;                        // this lane's query
  const bool q_ok = i_q < n;
  // the state's rows, and the values
  const float* st = a.states + (size_t)blockIdx.x * ((size_t)a.H * a.dv * a.DP) + (size_t)hd * a.dv * a.DP;
  for (int task = threadIdx.x; task < VB * (KD / 8); task += VH * 256) {
    const int g = task % (KD / 8), r = task / (KD / 8);
    float x[8];
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      float4 f = float4{0.f, 0.f, 0.f, 0.f};
      if (v0 + r < a.dv && 8 * g + 4 * u < a.DP)
        f = *(const float4*)(st + (size_t)(v0 + r) * a.DP + 8 * g + 4 * u);
      x[4 * u] = f.x; x[4 * u + 1] = f.y; x[4 * u + 2] = f.z; x[4 * u + 3] = f.w;
    }
    uint32_t h[4], l[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) h[i] = fc_pack(x[2 * i], x[2 * i + 1], l[i]);
    const int at = fc_row<KD>(r, g);
    *(uint4*)(xh + at) = make_uint4(h[0], h[1], h[2], h[3]);
    *(uint4*)(xl + at) = make_uint4(l[0], l[1], l[2], l[3]);
  }
  fc_stage_values<VB>(vt, v, rows.v_stride, hd, a.dv, v0, t0, n, rows.silu, a.wide);
  // the wave's queries, channels 16 i + 8 hl .. of every i
  fc_u32x4_t qh[KD / 16], ql[KD / 16];
  {
    const size_t row = (size_t)(t0 + (q_ok ? i_q : 0));
    const float2* tab = rows.table != nullptr ? rows.table + row * rows.half : nullptr;
    const bf16_t* x = q + row * rows.q_stride + (size_t)hd * a.d;
#pragma unroll
    for (int i = 0; i < KD / 16; ++i) {
      float f[8];
      fc_turned8(x, 16 * i + 8 * hl, a.d, tab, rows.half, rows.silu, a.wide, f);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        uint32_t lo;
        qh[i][e] = fc_pack(q_ok ? f[2 * e] : 0.f, q_ok ? f[2 * e + 1] : 0.f, lo);
        ql[i][e] = lo;
      }
    }
  }
  __syncthreads();
  fc_f32x16_t acc[VW / 32];
#pragma unroll
  for (int j = 0; j < VW / 32; ++j) {
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[j][r] = 0.f;
#pragma unroll
    for (int i = 0; i < KD / 16; ++i) {
      const int at = fc_row<KD>(part * VW + 32 * j + c, 2 * i + hl);
      const fc_u32x4_t sh = *(const fc_u32x4_t*)(xh + at);
      const fc_u32x4_t sl = *(const fc_u32x4_t*)(xl + at);
      acc[j] = fc_mfma(sh, qh[i], acc[j]);
      acc[j] = fc_mfma(sh, ql[i], acc[j]);
      acc[j] = fc_mfma(sl, qh[i], acc[j]);
    }
    const float g = fc_pow(lg, i_q + 1);
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[j][r] *= g;
  }
  __syncthreads();                                   // the state's rows are read
  for (int task = threadIdx.x; task < FC_C * (KD / 8); task += VH * 256) {
    const int g = task % (KD / 8), t = task / (KD / 8);
    if (t >= n && t >= (n + 31) / 32 * 32) continue;  // (no wave reads those rows)
    float x[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = 0.f;
    if (t < n) {
      const size_t row = (size_t)(t0 + t);
      const float2* tab = rows.table != nullptr ? rows.table + row * rows.half : nullptr;
      fc_turned8(k + row * rows.k_stride + (size_t)hd * a.d, 8 * g, a.d, tab, rows.half, rows.silu,
                 a.wide, x);
    }
    uint32_t h[4], l[4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
      h[i] = fc_pack(x[2 * i] * rows.k_scale, x[2 * i + 1] * rows.k_scale, l[i]);
    const int at = fc_row<KD>(t, g);
    *(uint4*)(xh + at) = make_uint4(h[0], h[1], h[2], h[3]);
    *(uint4*)(xl + at) = make_uint4(l[0], l[1], l[2], l[3]);
  }
  __syncthreads();
  if (32 * qb >= n) return;                          // (no barrier follows)
  for (int kb = 0; kb <= qb; ++kb) {
    fc_f32x16_t sc;
#pragma unroll
    for (int r = 0; r < 16; ++r) sc[r] = 0.f;
#pragma unroll
    for (int i = 0; i < KD / 16; ++i) {
      const int at = fc_row<KD>(32 * kb + c, 2 * i + hl);
      const fc_u32x4_t h = *(const fc_u32x4_t*)(xh + at);
      const fc_u32x4_t l = *(const fc_u32x4_t*)(xl + at);
      sc = fc_mfma(h, qh[i], sc);
      sc = fc_mfma(h, ql[i], sc);
      sc = fc_mfma(l, qh[i], sc);
    }
    // sc[r]: key 8 (r / 4) + 4 hl + r % 4 of the block, this lane's query
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const int back = i_q - (32 * kb + 8 * (r / 4) + 4 * hl + r % 4);
      sc[r] = back >= 0 ? sc[r] * fc_pow(lg, back) : 0.f;
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      // the registers 8 t .. 8 t + 7: keys 16 t + {0..3, 8..11} + 4 hl, and V^T in that order
      fc_u32x4_t ph, pl;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        uint32_t lo;
        ph[e] = fc_pack(sc[8 * t + 2 * e], sc[8 * t + 2 * e + 1], lo);
        pl[e] = lo;
      }
#pragma unroll
      for (int j = 0; j < VW / 32; ++j) {
        const int row = part * VW + 32 * j + c;
        const uint2 a0 = *(const uint2*)(vt + fc_tr(row, 16 * kb + 8 * t + 2 * hl));
        const uint2 a1 = *(const uint2*)(vt + fc_tr(row, 16 * kb + 8 * t + 4 + 2 * hl));
        const fc_u32x4_t av = {a0.x, a0.y, a1.x, a1.y};
        acc[j] = fc_mfma(av, ph, acc[j]);
        acc[j] = fc_mfma(av, pl, acc[j]);
      }
    }
  }
  if (!q_ok) return;
  float* o = out + (size_t)(t0 + i_q) * ((size_t)a.H * a.dv) + (size_t)hd * a.dv;
#pragma unroll
  for (int j = 0; j < VW / 32; ++j)
#pragma unroll
    for (int r4 = 0; r4 < 4; ++r4) {
      const int col = v0 + part * VW + 32 * j + 8 * r4 + 4 * hl;
      if ((a.dv & 3) == 0) {
        if (col < a.dv)
          *(float4*)(o + col) = float4{acc[j][4 * r4], acc[j][4 * r4 + 1], acc[j][4 * r4 + 2],
                                       acc[j][4 * r4 + 3]};
      } else {
#pragma unroll
        for (int x = 0; x < 4; ++x)
          if (col + x < a.dv) o[col + x] = acc[j][4 * r4 + x];
      }
    }
}

// chunks [n_chunks][4] and firsts [n_long][3] (device, int32) list the chunks of the step's long
// sequences: chunk c of sequence chunks[c][0] holds the tokens chunks[c][1] .. + chunks[c][2] - 1
// (of the step), a sequence's chunks lie in order, all of FC_C tokens but its last; firsts: the
// sequence, its first chunk, how many.  states: scratch, float32 [n_chunks, H dv DP].
extern "C" int zf_fixed_decay_chunks(const void* q, long long q_stride, const void* k,
                                     long long k_stride, const void* v, long long v_stride,
                                     const float* table, int half, int silu, float k_scale,
                                     const float* log2g, float* state, long long slot_stride,
                                     const int* state_slots, const int* chunks, int n_chunks,
                                     const int* firsts, int n_long, float* states, float* out,
                                     int H, int d, int dv, hipStream_t stream) {
  if (n_chunks <= 0 || n_long <= 0) return 0;
  const int DP = (d + 3) / 4 * 4;
  if (H <= 0 || d <= 0 || dv <= 0 || DP > 256 || slot_stride < (long long)H * dv * DP ||
      slot_stride % 4 != 0 || 2 * half > d || states == nullptr ||
      (table != nullptr && half <= 0))
    return -2;
  FixedDecayRows rows;
  rows.q_stride = q_stride; rows.k_stride = k_stride; rows.v_stride = v_stride;
  rows.table = (const float2*)table; rows.half = half; rows.silu = silu; rows.k_scale = k_scale;
  FixedDecayChunks a;
  a.chunks = chunks; a.firsts = firsts; a.log2g = log2g; a.states = states;
  a.H = H; a.d = d; a.dv = dv; a.DP = DP;
  a.wide = d % 8 == 0 && dv % 8 == 0 && q_stride % 8 == 0 && k_stride % 8 == 0 &&
           v_stride % 8 == 0 && (uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 &&
           (uintptr_t)v % 16 == 0 && (table == nullptr || (half % 8 == 0 && (uintptr_t)table % 16 == 0));
  const bf16_t *qp = (const bf16_t*)q, *kp = (const bf16_t*)k, *vp = (const bf16_t*)v;
  const long long quads = (long long)H * dv * DP / 4;
#define FC_RUN(KD, VB, NW, VH)                                                                    \
  {                                                                                              \
    const dim3 grid(n_chunks, H, (dv + VB - 1) / VB);                                            \
    hipLaunchKernelGGL((fixed_decay_sums_kernel<KD, VB, NW>), grid, dim3(NW * 64), 0, stream,    \
                       kp, vp, rows, a);                                                         \
    hipLaunchKernelGGL(fixed_decay_states_kernel, dim3((unsigned)((quads + 255) / 256), n_long), \
                       dim3(256), 0, stream, a, state, slot_stride, state_slots);                \
    hipLaunchKernelGGL((fixed_decay_outputs_kernel<KD, VB, VH>), grid, dim3(VH * 256), 0, stream,\
                       qp, kp, vp, rows, a, out);                                                \
  }
#define FC_RUN_VB(KD)                                                                            \
  if (dv <= 32) FC_RUN(KD, 32, 4, 1)                                                             \
  else if (dv <= 64) FC_RUN(KD, 64, 4, 2)                                                        \
  else FC_RUN(KD, 128, 8, 2)
  if (d <= 32) { FC_RUN_VB(32) }
  else if (d <= 64) { FC_RUN_VB(64) }
  else if (d <= 128) { FC_RUN_VB(128) }
  else if (dv <= 32) FC_RUN(256, 32, 4, 1)
  else FC_RUN(256, 64, 8, 2)
  ZF_CHECK_LAUNCH();
}
