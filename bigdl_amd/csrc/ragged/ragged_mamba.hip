// Selective scan (Mamba's recurrence) of the ragged engine.  Per channel c and state n, with a step size per token and channel,
//     S_t = exp(d_t A) S_(t-1) + d_t x_t B_t,     y_t = sum_n S_t C_t + D x_t,     d_t = softplus(step logits + bias),
// A [C, N] negative, B and C rows of N numbers shared by all channels.  The output leaves as y * silu(z).  S float
// [slots, C, N]; step sizes, decays, state and sums are float whatever the activation type T is.
#include "ragged_common.h"

using namespace ragged;

struct SelScanArgs {
  const void* x;         // [T, ldx] of type T: the convolved inputs
  int64_t ldx;
  const float* dt;       // [T, C] step logits
  const float* dt_bias;  // [C]
  const void* bc;        // [T, ldbc] of type T: columns b0 .. b0 + N - 1 are B, c0 .. c0 + N - 1 are C
  int64_t ldbc;
  int b0, c0;
  const float* A;        // [C, N]: log2(e) times the decay rates
  const float* D;        // [C]
  const void* z;         // [T, ldz] of type T, columns z0 ..: gates
  int64_t ldz;
  int z0;
  float* state;          // [slots, C, N]
  void* out;             // [T, C] of type T, or null (only the end states are wanted)
  float* sum_dt;         // [B, C] or null: the sum of a sequence's step sizes
  int C, N;
  int keep_end;          // 1: the last state goes back to `state`
};

// A channel's N states are spread over R neighbouring lanes, NS in registers each (R NS >= N; states past N have A = B = C = 0
// and stay zero); a wavefront serves 64 / R channels, a workgroup four wavefronts.  B and C of a block of TB tokens are staged
// in LDS as float; step logits, inputs and gates of U tokens are requested one group ahead.  Grid: (channel blocks, sequences).
constexpr int SS_U = 4;

template <typename T, int NS>
__global__ __launch_bounds__(256) void selective_scan_kernel(SelScanArgs a, int R, int TB, Batch bt) {
  extern __shared__ __attribute__((aligned(16))) float smem[];       // B [TB][R NS], C [TB][R NS]
  const int b = blockIdx.y, wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int r = lane % R, c = blockIdx.x * (256 / R) + wave * (64 / R) + lane / R;
  const bool ok = c < a.C;
  const int cc = ok ? c : a.C - 1;
  const int start = bt.seq_start[b], n = bt.seq_start[b + 1] - start, past = bt.seq_past[b], slot = bt.seq_slot[b];
  const int NP = R * NS;
  float S[NS], A[NS];
  float* sp = a.state + ((int64_t)slot * a.C + cc) * a.N;
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const int k = r * NS + i, kk = k < a.N ? k : a.N - 1;
    const float s = past > 0 ? sp[kk] : 0.f, d = a.A[(int64_t)cc * a.N + kk];
    S[i] = k < a.N ? s : 0.f;
    A[i] = k < a.N ? d : 0.f;
  }
  const float bias = a.dt_bias[cc], Dc = a.D[cc];
  const T* X = (const T*)a.x + cc;
  const T* Z = (const T*)a.z + a.z0 + cc;
  const T* BC = (const T*)a.bc;
  const float* DT = a.dt + cc;
  const bool outs = a.out != nullptr;
  float dn[SS_U], xn[SS_U], zn[SS_U], total = 0.f;
  auto request = [&](int i0) {
#pragma unroll
    for (int u = 0; u < SS_U; ++u) {
      const int64_t t = start + (i0 + u < n ? i0 + u : n - 1);
      dn[u] = DT[t * a.C];
      xn[u] = to_f(X[t * a.ldx]);
      zn[u] = outs ? to_f(Z[t * a.ldz]) : 0.f;
    }
  };
  if (n > 0) request(0);
  for (int j0 = 0; j0 < n; j0 += TB) {
    const int nt = n - j0 < TB ? n - j0 : TB;
    __syncthreads();                                         // the previous block has been read
    for (int e = threadIdx.x; e < nt * NP; e += 256) {
      const int tk = e / NP, k = e - tk * NP;
      const T* row = BC + (int64_t)(start + j0 + tk) * a.ldbc;
      smem[e] = k < a.N ? to_f(row[a.b0 + k]) : 0.f;
      if (outs) smem[TB * NP + e] = k < a.N ? to_f(row[a.c0 + k]) : 0.f;
    }
    __syncthreads();
    for (int i0 = 0; i0 < nt; i0 += SS_U) {
      float dc[SS_U], xc[SS_U], zc[SS_U];
#pragma unroll
      for (int u = 0; u < SS_U; ++u) { dc[u] = dn[u]; xc[u] = xn[u]; zc[u] = zn[u]; }
      if (j0 + i0 + SS_U < n) request(j0 + i0 + SS_U);
#pragma unroll
      for (int u = 0; u < SS_U; ++u) {
        if (i0 + u >= nt) break;
        const float raw = dc[u] + bias;
        const float d = fmaxf(raw, 0.f) + log1pf(__expf(-fabsf(raw)));
        total += d;
        const float dx = d * xc[u];
        const float4* b4 = reinterpret_cast<const float4*>(smem + (i0 + u) * NP + r * NS);
        const float4* c4 = reinterpret_cast<const float4*>(smem + (TB + i0 + u) * NP + r * NS);
        float y = 0.f, y2 = 0.f;
#pragma unroll
        for (int k = 0; k < NS / 4; ++k) {
          const float4 bb = b4[k];
          S[4 * k] = __builtin_amdgcn_exp2f(d * A[4 * k]) * S[4 * k] + dx * bb.x;
          S[4 * k + 1] = __builtin_amdgcn_exp2f(d * A[4 * k + 1]) * S[4 * k + 1] + dx * bb.y;
          S[4 * k + 2] = __builtin_amdgcn_exp2f(d * A[4 * k + 2]) * S[4 * k + 2] + dx * bb.z;
          S[4 * k + 3] = __builtin_amdgcn_exp2f(d * A[4 * k + 3]) * S[4 * k + 3] + dx * bb.w;
          if (outs) {
            const float4 q = c4[k];
            y += S[4 * k] * q.x + S[4 * k + 1] * q.y;
            y2 += S[4 * k + 2] * q.z + S[4 * k + 3] * q.w;
          }
        }
        if (outs) {
          y = group_sum(y + y2, R) + Dc * xc[u];
          if (r == 0 && ok) ((T*)a.out)[(int64_t)(start + j0 + i0 + u) * a.C + c] = from_f<T>(y * (zc[u] / (1.0f + __expf(-zc[u]))));
        }
      }
    }
  }
  if (!ok) return;
  if (a.sum_dt && r == 0) a.sum_dt[(int64_t)b * a.C + c] = total;
  if (a.keep_end) {
#pragma unroll
    for (int i = 0; i < NS; ++i)
      if (r * NS + i < a.N) sp[r * NS + i] = S[i];
  }
}

// ns: states per lane, 4, 8 or 16
extern "C" int ragged_selective_scan(SelScanArgs a, Batch bt, int ns, int dtype, hipStream_t st) {
  if (bt.B <= 0 || bt.B > 65535 || a.C <= 0 || a.N <= 0 || !a.x || !a.dt || !a.dt_bias || !a.bc || !a.A || !a.D || !a.state) return -1;
  if ((ns != 4 && ns != 8 && ns != 16) || a.N > 64 * ns || (a.out && !a.z) || a.b0 < 0 || a.c0 < 0) return -1;
  if (a.ldx < a.C || a.ldbc < a.b0 + a.N || a.ldbc < a.c0 + a.N || (a.out && a.ldz < a.z0 + a.C)) return -1;
  int R = 1;
  while (R * ns < a.N) R <<= 1;
  int TB = 4096 / (R * ns);                                  // at most 32 KB of LDS
  TB = TB > 32 ? 32 : TB;
  const size_t sm = 2 * (size_t)TB * R * ns * sizeof(float);
  const dim3 grid((a.C + 256 / R - 1) / (256 / R), bt.B);
  RAGGED_DISPATCH(dtype,
    if (ns == 4) hipLaunchKernelGGL((selective_scan_kernel<T, 4>), grid, dim3(256), sm, st, a, R, TB, bt);
    else if (ns == 8) hipLaunchKernelGGL((selective_scan_kernel<T, 8>), grid, dim3(256), sm, st, a, R, TB, bt);
    else hipLaunchKernelGGL((selective_scan_kernel<T, 16>), grid, dim3(256), sm, st, a, R, TB, bt))
  return RAGGED_LAUNCH_OK();
}

// Long portions are cut into chunks that are scanned side by side from zero.  A chunk's decay is exp(A times the sum of its
// step sizes), so the state at every chunk's start follows as S <- exp(A sum) S + local end state: one thread per state
// element walks a sequence's chunks, replaces the chunk's local end state in `chunks` [chunks, C, N] by its start state and
// leaves the last state in the sequence's slot.  cfirst[b] .. cfirst[b + 1] - 1 are b's chunks.
__global__ __launch_bounds__(256) void selective_chain_kernel(float* __restrict__ state, float* __restrict__ chunks,
                                                              const float* __restrict__ sum_dt, const float* __restrict__ A,
                                                              const int* __restrict__ cfirst, const int* __restrict__ seq_past,
                                                              const int* __restrict__ seq_slot, int C, int N) {
  const int b = blockIdx.y;
  const int64_t E = (int64_t)C * N, e = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= E) return;
  const int ch = (int)(e / N);
  const float rate = A[e];
  float* sp = state + (int64_t)seq_slot[b] * E + e;
  float S = seq_past[b] > 0 ? *sp : 0.f;
  const int c1 = cfirst[b + 1];
  for (int c0 = cfirst[b]; c0 < c1; c0 += 4) {
    float loc[4], dec[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int c = c0 + u < c1 ? c0 + u : c1 - 1;
      loc[u] = chunks[(int64_t)c * E + e];
      dec[u] = sum_dt[(int64_t)c * C + ch];
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (c0 + u < c1) {
        chunks[(int64_t)(c0 + u) * E + e] = S;
        S = __builtin_amdgcn_exp2f(rate * dec[u]) * S + loc[u];
      }
    }
  }
  *sp = S;
}

extern "C" int ragged_selective_chain(float* state, float* chunks, const float* sum_dt, const float* A, const int* cfirst,
                                      const int* seq_past, const int* seq_slot, int B, int C, int N, hipStream_t st) {
  if (B <= 0 || B > 65535 || C <= 0 || N <= 0) return -1;
  const int64_t E = (int64_t)C * N;
  hipLaunchKernelGGL(selective_chain_kernel, dim3((unsigned)((E + 255) / 256), B), dim3(256), 0, st, state, chunks, sum_dt, A, cfirst,
                     seq_past, seq_slot, C, N);
  return RAGGED_LAUNCH_OK();
}
