// State space recurrence (Mamba-2) over long bfloat16 portions on the matrix cores (v_mfma_f32_16x16x32_bf16), same semantics as
// the token-by-token scan in ragged_delta.hip:
//     S_t = exp(-a d_t) S_(t-1) + d_t B_t x_t^T,     y_t = S_t^T C_t + D x_t,     d_t = softplus(step logit + bias).
// One decay per token and head makes a block of 64 tokens a few products.  With L_t the sum of -a d over the block up to t,
//     y_t = exp(L_t) S_0^T C_t + sum_(s <= t) M[t, s] x_s,      M[t, s] = (C_t . B_s) exp(L_t - L_s) d_s  (+ D where s = t),
//     S_64 = exp(L_64) S_0 + sum_s B_s (exp(L_64 - L_s) d_s x_s)^T,
// every exponent being a difference that is not positive.  L is summed in 64 bits and kept as two floats: behind tokens with large
// steps a difference of two long sums would have lost the small decays in it.
//
//  * workgroup = one head of one sequence and 64 value columns; it walks the portion's blocks with the state in registers.  Wavefront
//    w owns columns 16 w .. 16 w + 15 of the state: float accumulators S[n][p] (lane = column p, four rows n per 16-row tile).
//  * those accumulators are, two tiles at a time, already laid out as the operand of the read-out S^T C (rows of a 32-row step in the
//    order 4 g + j, 16 + 4 g + j; the other operand is read in the same order), and the scores C B^T of a block, computed
//    transposed, are laid out as the operand of M x.  No float number passes through LDS.
//  * what is 32-bit stays so up to the matrix core: S, M and the weighted inputs go through it as two bfloat16 terms each (the upper
//    16 bits and the upper 16 bits of the exact remainder, 2^-16 relative); B, C and x are bfloat16 to begin with.
//  * rows of B and C, and B transposed, are staged in LDS by the whole workgroup from registers requested one block ahead; the score
//    tiles are shared out over the wavefronts (wavefront w: the 16 tokens 16 w ..) and exchanged through LDS.
// Tokens behind a portion's end take d = 0: they decay nothing and write nothing.
// A long portion is cut into segments that are walked side by side: first from zero for their end states alone (`out` null: no C,
// no scores), then, once space_chain_kernel has turned those into start states, for the outputs.
#include "ragged_space.h"

using namespace ragged;

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

union Frag {
  bf16x8 v;
  uint32_t u[4];
  uint16_t h[8];
  uint4 q;
  uint2 d2[2];
};

constexpr int SP_Q = 64;                                     // tokens of a block
constexpr int SP_LDT = SP_Q + 8;                             // halves of a row of B^T

// p0, p1 as the u-th pair of the two-term operand (hi, lo)
__device__ __forceinline__ void split_pair(float p0, float p1, Frag& hi, Frag& lo, int u) {
  const uint32_t h0 = __float_as_uint(p0) & 0xffff0000u, h1 = __float_as_uint(p1) & 0xffff0000u;
  const uint32_t l0 = __float_as_uint(p0 - __uint_as_float(h0)), l1 = __float_as_uint(p1 - __uint_as_float(h1));
  hi.u[u] = (h0 >> 16) | h1;
  lo.u[u] = (l0 >> 16) | (l1 & 0xffff0000u);
}

template <int KS> struct SpaceLds {
  static constexpr int LDN = 32 * KS + 8;                    // halves of a row of B or C
  static constexpr size_t rows = (size_t)SP_Q * LDN * 2, bt = (size_t)32 * KS * SP_LDT * 2;
  static constexpr size_t frags = 4 * 2 * 2 * 64 * sizeof(uint4), scal = 4 * 3 * SP_Q * sizeof(float);
  static constexpr size_t bytes = 2 * rows + bt + frags + scal;
};

// KS: 32-row steps of the state, N <= 32 KS (rows past N are zeros)
template <int KS>
__global__ __launch_bounds__(256, KS <= 4 ? 2 : 1) void state_space_mfma_kernel(SpaceArgs ss, const bf16* __restrict__ X, int64_t ldx, int G,
                                                               float* __restrict__ state, float* __restrict__ out, int H, int N, int vd,
                                                               Batch bt) {
  typedef SpaceLds<KS> L;
  constexpr int LDN = L::LDN, NT = 2 * KS;
  extern __shared__ __attribute__((aligned(16))) char sp_lds[];
  uint16_t* Cs = reinterpret_cast<uint16_t*>(sp_lds);                       // [token][n]
  uint16_t* Bs = reinterpret_cast<uint16_t*>(sp_lds + L::rows);
  uint16_t* BT = reinterpret_cast<uint16_t*>(sp_lds + 2 * L::rows);         // [n][token]
  uint4* Mf = reinterpret_cast<uint4*>(sp_lds + 2 * L::rows + L::bt);       // [token tile][32-token step][hi, lo][lane]
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lq = lane & 15, g4 = lane >> 4;
  float* cum = reinterpret_cast<float*>(sp_lds + 2 * L::rows + L::bt + L::frags) + wave * 3 * SP_Q;      // this wavefront's copy
  float* cuml = cum + SP_Q;                                  // (L = cum + cuml)
  float* dts = cum + 2 * SP_Q;
  const int h = blockIdx.y, b = blockIdx.z, g = h / (H / G);
  const int start = bt.seq_start[b], n = bt.seq_start[b + 1] - start, past = bt.seq_past[b], slot = bt.seq_slot[b];
  const int p = blockIdx.x * 64 + 16 * wave + lq, pc = p < vd ? p : vd - 1;
  const float rate = ss.rate[h], dtb = ss.dt_bias[h], skip = ss.D[h];
  const bool outs = out != nullptr;
  double total = 0.0;
  float* sp = state + ((int64_t)slot * H + h) * N * vd;
  f32x4 S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 16 * t + 4 * g4 + i;
      const float v = sp[(int64_t)(row < N ? row : N - 1) * vd + pc];       // no condition around the load
      S[t][i] = (past > 0 && row < N) ? v : 0.f;
    }

  Frag creg[KS], breg[KS], xn[2];
  float dtn = 0.f;
  auto fetch = [&](int c0) {                                 // the block's rows: lane = token for B, C and the step logits
    const int row = c0 + lane < n ? c0 + lane : n - 1;
    const bf16* src = X + (int64_t)(start + row) * ldx + g * N;
#pragma unroll
    for (int it = 0; it < KS; ++it) {
      const int e0 = 8 * (4 * it + wave);
      const bool in = e0 < N;                                // (N is a multiple of 8)
      creg[it].q = in && outs ? *reinterpret_cast<const uint4*>(src + ss.c0 + e0) : uint4{0, 0, 0, 0};
      breg[it].q = in ? *reinterpret_cast<const uint4*>(src + ss.b0 + e0) : uint4{0, 0, 0, 0};
    }
    dtn = to_f(((const bf16*)ss.dt)[(int64_t)(start + row) * ss.lddt + h]);
#pragma unroll
    for (int k = 0; k < 2; ++k)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int s = c0 + 32 * k + 16 * (j >> 2) + 4 * g4 + (j & 3);
        xn[k].h[j] = X[(int64_t)(start + (s < n ? s : n - 1)) * ldx + h * vd + pc].b;
      }
  };
  auto pieces = [&](const uint16_t* row, int ks) {           // 8 channels of a 32-channel step in the accumulators' order
    Frag f;
    f.d2[0] = *reinterpret_cast<const uint2*>(row + 32 * ks + 4 * g4);
    f.d2[1] = *reinterpret_cast<const uint2*>(row + 32 * ks + 16 + 4 * g4);
    return f;
  };
  if (n > 0) fetch(0);
  for (int c0 = 0; c0 < n; c0 += SP_Q) {
    const int nt = n - c0 < SP_Q ? n - c0 : SP_Q;
    __syncthreads();                                         // the previous block's rows and scores have been read
#pragma unroll
    for (int it = 0; it < KS; ++it) {
      const int e0 = 8 * (4 * it + wave);
      if (outs) {
        *reinterpret_cast<uint4*>(Cs + lane * LDN + e0) = creg[it].q;
        *reinterpret_cast<uint4*>(Bs + lane * LDN + e0) = breg[it].q;
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) BT[(e0 + u) * SP_LDT + lane] = breg[it].h[u];
    }
    Frag xs[2];
    xs[0].q = xn[0].q;
    xs[1].q = xn[1].q;
    // step sizes and the running sum of their decays, lane = token
    const float d = lane < nt ? softplusf_(dtn + dtb) : 0.f;
    double run = -(double)rate * d;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double below = __shfl_up(run, o, 64);
      run += lane >= o ? below : 0.0;
    }
    const float run_hi = (float)run, run_lo = (float)(run - (double)run_hi);
    cum[lane] = run_hi;
    cuml[lane] = run_lo;
    dts[lane] = d;
    total += run;                                            // (of lane 63: the whole block)
    const float last = lane_value(run_hi, 63), last_lo = lane_value(run_lo, 63);
    __syncthreads();
    if (c0 + SP_Q < n) fetch(c0 + SP_Q);                     // in flight during this block's arithmetic

    if (outs) {
      // ---- scores of this wavefront's 16 tokens t against the tokens s <= t, decayed, as two-term operands
      {
        const int t = 16 * wave + lq;
        const float ct = cum[t], ctl = cuml[t];
        Frag cf[KS];
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) cf[ks] = pieces(Cs + t * LDN, ks);
#pragma unroll
        for (int k = 0; k < 2; ++k) {
          if (2 * k > wave) continue;                          // (no token of these 32 lies at or before t)
          Frag hi, lo;
#pragma unroll
          for (int half = 0; half < 2; ++half) {
            const int st = 2 * k + half;
            f32x4 m = f32x4{0.f, 0.f, 0.f, 0.f};
            if (st <= wave) {
#pragma unroll
              for (int ks = 0; ks < KS; ++ks)
                m = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pieces(Bs + (16 * st + lq) * LDN, ks).v, cf[ks].v, m, 0, 0, 0);
              const int s0 = 16 * st + 4 * g4;
              const float4 cs = *reinterpret_cast<const float4*>(cum + s0), cl = *reinterpret_cast<const float4*>(cuml + s0);
              const float4 ds = *reinterpret_cast<const float4*>(dts + s0);
              const float cv[4] = {cs.x, cs.y, cs.z, cs.w}, lv[4] = {cl.x, cl.y, cl.z, cl.w}, dv[4] = {ds.x, ds.y, ds.z, ds.w};
#pragma unroll
              for (int i = 0; i < 4; ++i) {
                const int s = s0 + i;
                const float v = m[i] * __expf((ct - cv[i]) + (ctl - lv[i])) * dv[i];
                m[i] = s < t ? v : s == t ? v + skip : 0.f;
              }
            }
            split_pair(m[0], m[1], hi, lo, 2 * half);
            split_pair(m[2], m[3], hi, lo, 2 * half + 1);
          }
          Mf[((wave * 2 + k) * 2) * 64 + lane] = hi.q;
          Mf[((wave * 2 + k) * 2 + 1) * 64 + lane] = lo.q;
        }
      }
      // ---- what the block's start state adds to every token's output: y^T[p][t], lane = token t
      f32x4 Y[4];
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) Y[tt] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (past > 0 || c0 > 0) {
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
          Frag hi, lo;
#pragma unroll
          for (int half = 0; half < 2; ++half) {
            split_pair(S[2 * ks + half][0], S[2 * ks + half][1], hi, lo, 2 * half);
            split_pair(S[2 * ks + half][2], S[2 * ks + half][3], hi, lo, 2 * half + 1);
          }
#pragma unroll
          for (int tt = 0; tt < 4; ++tt) {
            const Frag cf = pieces(Cs + (16 * tt + lq) * LDN, ks);
            Y[tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(hi.v, cf.v, Y[tt], 0, 0, 0);
            Y[tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lo.v, cf.v, Y[tt], 0, 0, 0);
          }
        }
#pragma unroll
        for (int tt = 0; tt < 4; ++tt) Y[tt] *= expf(cum[16 * tt + lq]);
      }
      __syncthreads();                                         // every wavefront's scores are there
      // ---- the block's own tokens
#pragma unroll
      for (int tt = 0; tt < 4; ++tt) {
#pragma unroll
        for (int k = 0; k < 2; ++k) {
          if (2 * k > tt) continue;
          Frag hi, lo;
          hi.q = Mf[((tt * 2 + k) * 2) * 64 + lane];
          lo.q = Mf[((tt * 2 + k) * 2 + 1) * 64 + lane];
          Y[tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xs[k].v, hi.v, Y[tt], 0, 0, 0);
          Y[tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(xs[k].v, lo.v, Y[tt], 0, 0, 0);
        }
        const int t = 16 * tt + lq, p0 = blockIdx.x * 64 + 16 * wave + 4 * g4;
        if (t < nt) {
          float* o = out + (int64_t)(start + c0 + t) * (H * vd) + h * vd + p0;
          if ((vd & 3) == 0) {
            if (p0 < vd) *reinterpret_cast<float4*>(o) = float4{Y[tt][0], Y[tt][1], Y[tt][2], Y[tt][3]};
          } else {
#pragma unroll
            for (int i = 0; i < 4; ++i)
              if (p0 + i < vd) o[i] = Y[tt][i];
          }
        }
      }
    }
    // ---- the state behind the block: decayed, plus the inputs weighted by what is left of them at the block's end
    Frag whi[2], wlo[2];
#pragma unroll
    for (int k = 0; k < 2; ++k)
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const int s0 = 32 * k + 16 * half + 4 * g4;
        const float4 cs = *reinterpret_cast<const float4*>(cum + s0), cl = *reinterpret_cast<const float4*>(cuml + s0);
        const float4 ds = *reinterpret_cast<const float4*>(dts + s0);
        const float cv[4] = {cs.x, cs.y, cs.z, cs.w}, lv[4] = {cl.x, cl.y, cl.z, cl.w}, dv[4] = {ds.x, ds.y, ds.z, ds.w};
        float w[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) w[i] = __expf((last - cv[i]) + (last_lo - lv[i])) * dv[i] * __uint_as_float((uint32_t)xs[k].h[4 * half + i] << 16);
        split_pair(w[0], w[1], whi[k], wlo[k], 2 * half);
        split_pair(w[2], w[3], whi[k], wlo[k], 2 * half + 1);
      }
    const float all = expf(last);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      S[t] *= all;
#pragma unroll
      for (int k = 0; k < 2; ++k) {
        const Frag bf = pieces(BT + (16 * t + lq) * SP_LDT, k);
        S[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf.v, whi[k].v, S[t], 0, 0, 0);
        S[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(bf.v, wlo[k].v, S[t], 0, 0, 0);
      }
    }
  }
  if (ss.sum_log && blockIdx.x == 0 && threadIdx.x == 63) ss.sum_log[(int64_t)b * H + h] = (float)total;
  if (p >= vd || !ss.keep_end) return;
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = 16 * t + 4 * g4 + i;
      if (row < N) sp[(int64_t)row * vd + p] = S[t][i];
    }
}

// 1 when the kernel serves these sizes (bfloat16 only; b0, c0 and ldx of the inputs' matrix must be multiples of 8 as well)
extern "C" int ragged_state_space_mfma_ok(int N) { return N > 0 && N % 8 == 0 && N <= 256; }

template <int KS>
static int launch_space(SpaceArgs ss, const void* X, int64_t ldx, int G, float* state, float* out, int H, int N, int vd, Batch bt, hipStream_t st) {
  constexpr size_t lds = SpaceLds<KS>::bytes;
  if (lds > 64 * 1024) {                                     // (asked for once per process and kernel)
    static const hipError_t asked = hipFuncSetAttribute(reinterpret_cast<const void*>(state_space_mfma_kernel<KS>),
                                                        hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (asked != hipSuccess) return -3;
  }
  hipLaunchKernelGGL(state_space_mfma_kernel<KS>, dim3((vd + 63) / 64, H, bt.B), dim3(256), lds, st, ss, (const bf16*)X, ldx, G, state, out, H,
                     N, vd, bt);
  return RAGGED_LAUNCH_OK();
}

extern "C" int ragged_state_space_mfma(SpaceArgs ss, const void* X, int64_t ldx, int G, float* state, float* out, int H, int N, int vd,
                                       Batch bt, hipStream_t st) {
  if (bt.B <= 0 || bt.B > 65535 || H <= 0 || H > 65535 || vd <= 0 || G <= 0 || H % G || !ragged_state_space_mfma_ok(N)) return -1;
  if (!ss.dt || !ss.dt_bias || !ss.rate || !ss.D || ss.lddt < H || ss.b0 < 0 || ss.c0 < 0 || !X || !state || (!out && !ss.keep_end)) return -1;
  if (ss.b0 % 8 || ss.c0 % 8 || ldx % 8 || (uintptr_t)X % 16 || (uintptr_t)out % 16) return -1;
  if (ldx < (int64_t)H * vd || ldx < ss.b0 + (int64_t)G * N || ldx < ss.c0 + (int64_t)G * N) return -1;
#define SP_CASE(KS) return launch_space<KS>(ss, X, ldx, G, state, out, H, N, vd, bt, st)
  if (N <= 32) SP_CASE(1);
  if (N <= 64) SP_CASE(2);
  if (N <= 96) SP_CASE(3);
  if (N <= 128) SP_CASE(4);
  SP_CASE(8);
#undef SP_CASE
}

// The walk over a sequence's segments: one thread per four neighbouring state elements replaces a segment's local end state in
// `segs` [segments, H, N, vd] by its start state and leaves the last state in the sequence's slot.  A segment's decay is one number per
// head, exp(sum_log[segment, h]).  cfirst[b] .. cfirst[b + 1] - 1 are b's segments.  V: elements per thread (a head has V * k).
template <int V>
__global__ __launch_bounds__(256) void space_chain_kernel(float* __restrict__ state, float* __restrict__ segs, const float* __restrict__ sum_log,
                                                          const int* __restrict__ cfirst, const int* __restrict__ seq_past,
                                                          const int* __restrict__ seq_slot, int H, int per_head) {
  const int b = blockIdx.y;
  const int64_t E = (int64_t)H * per_head, e = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V;
  if (e >= E) return;
  const int h = (int)(e / per_head);
  float* sp = state + (int64_t)seq_slot[b] * E + e;
  float S[V];
#pragma unroll
  for (int i = 0; i < V; ++i) S[i] = seq_past[b] > 0 ? sp[i] : 0.f;
  const int c1 = cfirst[b + 1];
  for (int c0 = cfirst[b]; c0 < c1; c0 += 4) {
    float loc[4][V], dec[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = c0 + u < c1 ? c0 + u : c1 - 1;
      if (V == 4) {
        const float4 q = *reinterpret_cast<const float4*>(segs + (int64_t)c * E + e);
        loc[u][0] = q.x; loc[u][1 % V] = q.y; loc[u][2 % V] = q.z; loc[u][3 % V] = q.w;
      } else {
        loc[u][0] = segs[(int64_t)c * E + e];
      }
      dec[u] = sum_log[(int64_t)c * H + h];
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (c0 + u >= c1) break;
      float* o = segs + (int64_t)(c0 + u) * E + e;
      const float f = expf(dec[u]);
      if (V == 4) *reinterpret_cast<float4*>(o) = float4{S[0], S[1 % V], S[2 % V], S[3 % V]};
      else o[0] = S[0];
#pragma unroll
      for (int i = 0; i < V; ++i) S[i] = f * S[i] + loc[u][i];
    }
  }
#pragma unroll
  for (int i = 0; i < V; ++i) sp[i] = S[i];
}

extern "C" int ragged_space_chain(float* state, float* segs, const float* sum_log, const int* cfirst, const int* seq_past, const int* seq_slot,
                                  int B, int H, int N, int vd, hipStream_t st) {
  if (B <= 0 || B > 65535 || H <= 0 || N <= 0 || vd <= 0 || !state || !segs || !sum_log) return -1;
  const int64_t per_head = (int64_t)N * vd, E = per_head * H;
  if (per_head > 0x7fffffff) return -1;
  if (per_head % 4 == 0)
    hipLaunchKernelGGL(space_chain_kernel<4>, dim3((unsigned)((E / 4 + 255) / 256), B), dim3(256), 0, st, state, segs, sum_log, cfirst, seq_past,
                       seq_slot, H, (int)per_head);
  else
    hipLaunchKernelGGL(space_chain_kernel<1>, dim3((unsigned)((E + 255) / 256), B), dim3(256), 0, st, state, segs, sum_log, cfirst, seq_past,
                       seq_slot, H, (int)per_head);
  return RAGGED_LAUNCH_OK();
}
