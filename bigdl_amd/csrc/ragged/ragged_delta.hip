// Generalised delta rule of the ragged engine: a matrix state per head that decays per key channel, forgets along the
// direction of the unit key and then takes the new key / value pair,
//     S_t = diag(w_t) S_(t-1) - (a_t * n_t) (n_t^T S_(t-1)) + k_t v_t^T,     o_t = S_t^T r_t,     n = k / sqrt(|k|^2 + tiny)
// with both terms reading the old state.  S float [d, vd] per (slot, head).  Everything but the projections themselves
// (decay, removal rate, unit key, state, outputs) is float whatever the activation type T is.
// The gated delta rule is its relative with one decay g and one write strength beta per head,
//     S' = g S,   u = beta (v - S'^T k),   S <- S' + k u^T,   o = S^T q,     k, q unit vectors behind short convolutions:
// the same scan with two arrays and two scalars per token instead of five arrays, or with three where g has a number per key
// channel.  The state space recurrence (Mamba-2) is the one without the forgetting term,
//     S <- exp(-a d) S + d B x^T,   y = S^T C + D x,     d = softplus(step logit + bias) per head.
#include "ragged_space.h"

using namespace ragged;

// ---------------------------------------------------------------------------------------------------------------
// The scan's five arrays from this step's projections, float [rows, H d] each:
//   rf = r,  wf = exp(-rate * sigmoid(decay logits + w0)),  nf = n,  bf = sigmoid(a logits + ab) * n,  kf = k
// r, k and the a logits are columns of P (type T); the decay logits come from a second small product and are float.
// One wavefront per (row, head).
template <typename T>
__global__ __launch_bounds__(256) void delta_gates_kernel(const T* __restrict__ P, int64_t ldp, int r0, int k0, int a0,
                                                          const float* __restrict__ wl, const float* __restrict__ w0,
                                                          const float* __restrict__ ab, float rate, float tiny,
                                                          float* __restrict__ rf, float* __restrict__ wf, float* __restrict__ nf,
                                                          float* __restrict__ bf, float* __restrict__ kf, int64_t items, int H, int d) {
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= items) return;
  const int64_t t = item / H;
  const int h = (int)(item % H);
  const T* row = P + t * ldp;
  float ss = 0.f;
  for (int c = lane; c < d; c += 64) { const float k = to_f(row[k0 + h * d + c]); ss += k * k; }
  const float inv = 1.0f / sqrtf(wave_sum(ss) + tiny);
  for (int c = lane; c < d; c += 64) {
    const int ch = h * d + c;
    const int64_t o = t * (int64_t)(H * d) + ch;
    const float k = to_f(row[k0 + ch]), n = k * inv;
    const float sw = 1.0f / (1.0f + expf(-(wl[o] + w0[ch])));
    const float sa = 1.0f / (1.0f + expf(-(to_f(row[a0 + ch]) + ab[ch])));
    rf[o] = to_f(row[r0 + ch]);
    wf[o] = expf(-rate * sw);
    nf[o] = n;
    bf[o] = sa * n;
    kf[o] = k;
  }
}

extern "C" int ragged_delta_gates(const void* P, int64_t ldp, int r0, int k0, int a0, const float* wl, const float* w0,
                                  const float* ab, float rate, float tiny, float* rf, float* wf, float* nf, float* bf, float* kf,
                                  int64_t rows, int H, int d, int dtype, hipStream_t st) {
  if (rows <= 0 || H <= 0 || d <= 0 || rows * H > 0x7fffffff || r0 < 0 || k0 < 0 || a0 < 0) return -1;
  const int64_t items = rows * H;
  RAGGED_DISPATCH(dtype, hipLaunchKernelGGL((delta_gates_kernel<T>), dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, (const T*)P,
                                            ldp, r0, k0, a0, wl, w0, ab, rate, tiny, rf, wf, nf, bf, kf, items, H, d))
  return RAGGED_LAUNCH_OK();
}

// ---------------------------------------------------------------------------------------------------------------
// The gated delta rule's inputs from this step's projections (columns 0 .. of P: q [G d] | k [G d] | v [H vd], all of them
// behind a short causal convolution and silu): qf = unit(q) * d^(-1/2), kf = unit(k), float [rows, G d] each, with unit(u) =
// u / sqrt(|u|^2 + tiny); vo of type T [rows, H vd]; gb float [rows, H, 2] = (exp(-arate softplus(a + dt bias)), sigmoid(b)).
// With a decay per key channel: wf float [rows, H d] = exp(-arate_h softplus(wl + dt bias)), wl float logits, and gb = (1, sigmoid(b)).
// The inputs before this step come from `state` [slots, taps - 1, C]; `write_state` (every sequence brings exactly one row)
// also shifts it.  One wavefront per (block of rows, item): 2 G unit vectors, blocks
// of value channels, blocks of decay channels, the gates.
struct GatedDeltaArgs {
  const void* P;
  int64_t ldp;
  const float* cw;       // [C, taps], C = 2 G d + H vd
  int taps;
  void* state;
  int b0, a0;            // columns of P: write strengths and step logits, H each
  const float* arate;    // [H]
  const float* dt_bias;  // [H], or with wl [H d]
  float tiny;
  const float* wl;       // [rows, H d] or null: decay logits per key channel
  float* wf;             // [rows, H d]
  float* qf;
  float* kf;
  void* vo;
  float* gb;
  int H, G, d, vd, write_state;
};

// K: 64-channel pieces of an item (a unit vector's d <= 64 K); a lane holds one channel of each.  RB rows are walked with the
// last TAPS - 1 inputs in registers (TAPS = 0: any number of taps, every tap is read where it is needed).
template <typename T, int K, int TAPS>
__global__ __launch_bounds__(256) void gated_delta_prep_kernel(GatedDeltaArgs a, int items, int RB, Batch bt) {
  constexpr int M = TAPS > 1 ? TAPS - 1 : 1, W = TAPS > 0 ? TAPS : 1;
  const int lane = threadIdx.x & 63;
  // (the same for a whole wavefront: kept in scalar registers)
  const unsigned id = __builtin_amdgcn_readfirstlane(blockIdx.x * 4 + (threadIdx.x >> 6));
  const int t0 = (int)(id / (unsigned)items) * RB, it = (int)(id % (unsigned)items);
  if (t0 >= bt.T) return;
  const int t1 = t0 + RB < bt.T ? t0 + RB : bt.T;
  const T* P = (const T*)a.P;
  if (it == items - 1) {                                     // decays and write strengths
    for (int e = lane; e < (t1 - t0) * a.H; e += 64) {
      const int t = t0 + e / a.H, h = e % a.H;
      const T* row = P + (int64_t)t * a.ldp;
      float* o = a.gb + ((int64_t)t * a.H + h) * 2;
      o[0] = a.wl ? 1.f : expf(-a.arate[h] * softplusf_(to_f(row[a.a0 + h]) + a.dt_bias[h]));
      o[1] = 1.0f / (1.0f + expf(-to_f(row[a.b0 + h])));
    }
    return;
  }
  const int vitems = (a.H * a.vd + 64 * K - 1) / (64 * K);
  if (it >= 2 * a.G + vitems) {                              // decays per key channel
    const int HD = a.H * a.d, c0 = (it - 2 * a.G - vitems) * 64 * K + lane;
    float rate[K], bias[K];
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int c = c0 + 64 * k < HD ? c0 + 64 * k : HD - 1;
      rate[k] = a.arate[c / a.d];
      bias[k] = a.dt_bias[c];
    }
    for (int t = t0; t < t1; ++t) {
#pragma unroll
      for (int k = 0; k < K; ++k) {
        const int c = c0 + 64 * k;
        if (c < HD) a.wf[(int64_t)t * HD + c] = expf(-rate[k] * softplusf_(a.wl[(int64_t)t * HD + c] + bias[k]));
      }
    }
    return;
  }
  const int C = 2 * a.G * a.d + a.H * a.vd, taps = TAPS > 0 ? TAPS : a.taps, keep = taps - 1;
  const bool unit = it < 2 * a.G, isq = it < a.G;
  const int v0 = (it - 2 * a.G) * 64 * K;                    // a value item's first value channel
  const int ch0 = unit ? it * a.d : 2 * a.G * a.d + v0;
  const int width = unit ? a.d : (a.H * a.vd - v0 < 64 * K ? a.H * a.vd - v0 : 64 * K);
  T* S = (T*)a.state;
  auto input = [&](int t, int back, int pos, int past, int slot, int ch) -> T {      // (the address is chosen first)
    const int pp = pos - back;
    const T* p = P + (int64_t)t * a.ldp + ch;
    if (pp >= past) p -= back * a.ldp;
    else if (pp >= 0) p = S + ((int64_t)slot * keep + (pp - past + keep)) * C + ch;
    T v = *p;
    if (pp < 0) v = from_f<T>(0.f);
    return v;
  };
  int chs[K];
  float w[K][W];
  T hist[K][M];
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int c = lane + 64 * k;
    chs[k] = ch0 + (c < width ? c : width - 1);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[k][j] = a.cw[(int64_t)chs[k] * TAPS + j];
  }
  T next[K];                                                 // the row after the current one, requested early
#pragma unroll
  for (int k = 0; k < K; ++k) next[k] = P[(int64_t)t0 * a.ldp + chs[k]];
  // what belongs to the rows' sequence is looked up once per sequence (a batch's sequences lie one behind the other)
  int b = bt.tok_seq[t0], pos = bt.tok_pos[t0], past = bt.seq_past[b], slot = bt.seq_slot[b], end = bt.seq_start[b + 1];
  const float qscale = isq ? 1.0f / sqrtf((float)a.d) : 1.0f;
  for (int t = t0; t < t1; ++t, ++pos) {
    if (t == end) { ++b; pos = past = bt.seq_past[b]; slot = bt.seq_slot[b]; end = bt.seq_start[b + 1]; }
    float u[K], ss = 0.f;
    T row[K];
#pragma unroll
    for (int k = 0; k < K; ++k) {
      row[k] = next[k];
      next[k] = P[(int64_t)(t + 1 < t1 ? t + 1 : t) * a.ldp + chs[k]];
    }
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const T cur = row[k];
      u[k] = 0.f;
      const bool ok = lane + 64 * k < width;
      if (TAPS > 0) {
        if (TAPS > 1 && (t == t0 || pos == past)) {          // (the same branch for the whole wavefront)
#pragma unroll
          for (int j = 0; j < M; ++j) hist[k][j] = input(t, TAPS - 1 - j, pos, past, slot, chs[k]);
        }
        if (TAPS > 1) {
#pragma unroll
          for (int j = 0; j < M; ++j) u[k] += w[k][j] * to_f(hist[k][j]);
        }
        u[k] += w[k][W - 1] * to_f(cur);
        if (TAPS > 1) {
#pragma unroll
          for (int j = 0; j + 1 < M; ++j) hist[k][j] = hist[k][j + 1];
          hist[k][M - 1] = cur;
          if (a.write_state && ok) {
#pragma unroll
            for (int j = 0; j < M; ++j) S[((int64_t)slot * keep + j) * C + chs[k]] = hist[k][j];
          }
        }
      } else {
        for (int j = 0; j < taps; ++j) {
          const T raw = input(t, keep - j, pos, past, slot, chs[k]);
          u[k] += a.cw[(int64_t)chs[k] * taps + j] * to_f(raw);
          if (a.write_state && ok && j > 0) S[((int64_t)slot * keep + j - 1) * C + chs[k]] = raw;   // (row j - 1 has been read)
        }
      }
      u[k] = ok ? u[k] * sigmoidf_(u[k]) : 0.f;
      ss += u[k] * u[k];
    }
    if (unit) {
      const float f = qscale / sqrtf(wave_sum(ss) + a.tiny);
      float* o = (isq ? a.qf : a.kf) + ((int64_t)t * a.G + (isq ? it : it - a.G)) * a.d;
#pragma unroll
      for (int k = 0; k < K; ++k)
        if (lane + 64 * k < width) o[lane + 64 * k] = u[k] * f;
    } else {
      T* o = (T*)a.vo + (int64_t)t * a.H * a.vd + v0;
#pragma unroll
      for (int k = 0; k < K; ++k)
        if (lane + 64 * k < width) o[lane + 64 * k] = from_f<T>(u[k]);
    }
  }
}

template <typename T, int K>
static void launch_gated_prep(GatedDeltaArgs a, Batch bt, hipStream_t st) {
  const int items = 2 * a.G + (a.H * a.vd + 64 * K - 1) / (64 * K) + (a.wl ? (a.H * a.d + 64 * K - 1) / (64 * K) : 0) + 1;
  const int RB = bt.T >= 512 ? 8 : bt.T >= 64 ? 2 : 1;
  const int64_t waves = (int64_t)((bt.T + RB - 1) / RB) * items;
  const dim3 grid((unsigned)((waves + 3) / 4));
  if (a.taps == 4) hipLaunchKernelGGL((gated_delta_prep_kernel<T, K, 4>), grid, dim3(256), 0, st, a, items, RB, bt);
  else if (a.taps == 3) hipLaunchKernelGGL((gated_delta_prep_kernel<T, K, 3>), grid, dim3(256), 0, st, a, items, RB, bt);
  else hipLaunchKernelGGL((gated_delta_prep_kernel<T, K, 0>), grid, dim3(256), 0, st, a, items, RB, bt);
}

extern "C" int ragged_gated_delta_prep(GatedDeltaArgs a, Batch bt, int dtype, hipStream_t st) {
  if (bt.T <= 0 || a.H <= 0 || a.G <= 0 || a.H % a.G || a.d <= 0 || a.d > 1024 || a.vd <= 0 || a.taps < 1 || a.taps > 16) return -1;
  if (!a.P || !a.cw || (a.taps > 1 && !a.state) || !a.arate || !a.dt_bias || !a.qf || !a.kf || !a.vo || !a.gb) return -1;
  const int C = 2 * a.G * a.d + a.H * a.vd;
  if (a.b0 < C || a.ldp < a.b0 + a.H || (!a.wl && (a.a0 < C || a.ldp < a.a0 + a.H)) || (a.wl && !a.wf) || (a.write_state && bt.B != bt.T)) return -1;
  if ((int64_t)bt.T * (2 * a.G + a.H * (a.vd + a.d)) > 0x7fffffff) return -1;
  if (a.taps == 1) a.write_state = 0;
  RAGGED_DISPATCH(dtype,
    if (a.d <= 64) launch_gated_prep<T, 1>(a, bt, st);
    else if (a.d <= 128) launch_gated_prep<T, 2>(a, bt, st);
    else if (a.d <= 256) launch_gated_prep<T, 4>(a, bt, st);
    else launch_gated_prep<T, 16>(a, bt, st))
  return RAGGED_LAUNCH_OK();
}

// ---------------------------------------------------------------------------------------------------------------
// The scan.  Columns of S are independent: column j follows s <- w * s - b (n . s) + k v_j, and its output is r . s.
// A wavefront owns 64 / R columns; R neighbouring lanes share a column, lane r of them holds rows 16 r .. 16 r + 15 in
// registers (R = d / 16 rounded up to a power of two; rows past d carry w = 1 and zeros and stay zero), so a token costs
// two cross-lane sums of R partial products (DPP moves): n . s before the update, r . s after it.  A workgroup is NW such
// wavefronts (as many as the state has columns for, at most four: a wavefront without columns would still read all five
// arrays).  The five arrays of a block of TB tokens are brought into LDS by the whole workgroup with coalesced loads
// while the previous block is scanned (register look-ahead, two LDS buffers) and read back as 16-byte broadcasts.
// Grid: (column blocks, heads, sequences).  `values` = 0: v is taken as 0 (the state only decays and forgets: from an
// identity state this yields a chunk's transition matrix).  `trans`: both at once, sequences grid.z / 2 .. scan the same tokens
// without values from the d columns of `trans` (a state array like `state`).
// MODE: which recurrence.
//   general  five arrays, as above.
//   gated    q and k of G heads (head h reads head h / (H / G)); `gb` holds every token's decay and write strength per head, and the
//            four arrays of the general form shrink to k and scalars: w = g, n = k, b = beta g k, and k v takes the factor beta.
//   channel  the gated rule with a decay per key channel: q, k and the decays w of H heads; of `gb` only the write strength counts.
//   space    the state space recurrence: q and k are the rows C and B of G groups, columns c0 .. and b0 .. of P (type T); a token's
//            decay and step size per head come from its step logit (`ss`), the read-out takes D v on top.
enum DeltaMode { DL_GENERAL, DL_GATED, DL_CHANNEL, DL_SPACE };

constexpr int DL_DR = 16;
constexpr int DL_SEG = DL_DR + 4;   // LDS floats per lane group and token (padding shifts the banks between groups)
constexpr int DL_TBR = 64;          // TB * R <= this

template <typename T, int NW, int MODE>
__global__ __launch_bounds__(64 * NW, 2) void delta_scan_kernel(const float* __restrict__ rf, const float* __restrict__ wf,
                                                         const float* __restrict__ nf, const float* __restrict__ bf,
                                                         const float* __restrict__ kf, const float* __restrict__ gb, int G,
                                                         const T* __restrict__ P, int64_t ldp, int v0,
                                                         float* __restrict__ state, float* __restrict__ out, int H, int d, int vd,
                                                         float* __restrict__ trans, int R, int TB, int values, SpaceArgs ss, Batch bt) {
  constexpr int NA = MODE == DL_GENERAL ? 5 : MODE == DL_CHANNEL ? 3 : 2, KI = MODE == DL_GENERAL ? 4 : 1;    // arrays, k's place among them
  constexpr bool GB = MODE != DL_GENERAL;                    // two scalars per token
  constexpr int NT = 64 * NW, PRE = DL_TBR * DL_DR / NT;     // threads; elements of an array's block per thread
  extern __shared__ __attribute__((aligned(16))) float smem[];   // 2 x { r, w, n, b, k (r, k, w): [TB][R][SEG] each, v[TB][wcols], (g, beta)[TB] }
  int b = blockIdx.z;
  bool fresh = true;                                         // sequences without a past start from zero
  if (trans) {
    const int half = gridDim.z >> 1;
    if (b >= half) { b -= half; state = trans; vd = d; values = 0; fresh = false; }
  }
  const int h = blockIdx.y, tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63;
  const int cols = 64 / R, wcols = NW * cols;
  if ((int)blockIdx.x * wcols >= vd) return;                 // (the whole workgroup: no barrier is left waiting)
  const int r = lane % R, lc = wave * cols + lane / R;     // column inside the workgroup's block
  const int col = blockIdx.x * wcols + lc;
  const int start = bt.seq_start[b], n = bt.seq_start[b + 1] - start, past = bt.seq_past[b], slot = bt.seq_slot[b];
  const bool colok = col < vd;
  const int row0 = r * DL_DR;
  const int gh = GB ? h / (H / G) : h;                       // the head of q and k that this head reads
  const int HD = GB ? G * d : H * d, hd0 = gh * d;           // floats of an array's row, this head's first
  const int qsz = TB * R * DL_SEG;                         // floats of one array in a buffer
  const int bufsz = NA * qsz + TB * wcols + (GB ? (2 * TB + 3) & ~3 : 0);
  const float rate = MODE == DL_SPACE ? ss.rate[h] : 0.f, dtb = MODE == DL_SPACE ? ss.dt_bias[h] : 0.f, skip = MODE == DL_SPACE ? ss.D[h] : 0.f;
  float S[DL_DR];
  float* sp = state + (((int64_t)slot * H + h) * d) * vd;
  {
    const int cc = colok ? col : vd - 1;
#pragma unroll
    for (int k = 0; k < DL_DR; ++k) {
      const int row = row0 + k;
      const float v = sp[(unsigned)((row < d ? row : d - 1) * vd + cc)];    // no condition around the load
      S[k] = ((past > 0 || !fresh) && colok && row < d) ? v : 0.f;
    }
  }
  // A block's element e = (token tk, row): a token has R * 16 rows and a workgroup 2^lw columns, both powers of two, so no step
  // divides; tokens are the slow index, so a block of few tokens (a single decoded one) ends the loops early.  Every address is a
  // base that the workgroup shares plus a short offset.
  const int lr = 31 - __clz(R * DL_DR), rows = 1 << lr, lw = 31 - __clz(wcols);
  float pre[NA][PRE], prev[4], preg = 0.f;
  auto fetch = [&](int i0) {                               // block of tokens i0 .. i0 + TB - 1 into registers
    const int nt = n - i0 < TB ? n - i0 : TB;
    const int64_t t0 = start + i0;
    const T* prow = P + t0 * ldp;
#pragma unroll
    for (int u = 0; u < PRE; ++u) {
      if (NT * u >= nt << lr) break;
      const int e = tid + NT * u, tk = e >> lr, row = e & (rows - 1);
      const bool ok = tk < nt && row < d;
#pragma unroll
      for (int a = 0; a < NA; ++a) {
        float v;
        if (MODE == DL_SPACE) {
          v = to_f((prow + (a == 0 ? ss.c0 : ss.b0) + hd0)[ok ? (unsigned)(tk * (int)ldp + row) : 0u]);
        } else {
          const float* src = a == 0 ? rf : MODE == DL_CHANNEL && a == 2 ? wf : GB ? kf : a == 1 ? wf : a == 2 ? nf : a == 3 ? bf : kf;
          const int stride = MODE == DL_CHANNEL && a == 2 ? H * d : HD, first = MODE == DL_CHANNEL && a == 2 ? h * d : hd0;
          v = (src + t0 * stride + first)[ok ? (unsigned)(tk * stride + row) : 0u];
        }
        pre[a][u] = ok ? v : MODE == DL_GENERAL && a == 1 ? 1.f : 0.f;       // padding: w = 1, everything else 0
      }
    }
    if (GB && tid < 2 * TB && tid >> 1 < nt) {
      if (MODE == DL_SPACE) {
        const float step = softplusf_(to_f(((const T*)ss.dt)[(t0 + (tid >> 1)) * ss.lddt + h]) + dtb);
        preg = (tid & 1) ? step : expf(-rate * step);
      } else {
        preg = gb[((t0 + (tid >> 1)) * H + h) * 2 + (tid & 1)];
      }
    }
    if (!values) {
#pragma unroll
      for (int u = 0; u < 4; ++u) prev[u] = 0.f;
      return;
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (NT * u >= nt << lw) break;
      const int e = tid + NT * u, tk = e >> lw, c = blockIdx.x * wcols + (e & (wcols - 1));
      const bool ok = tk < nt && c < vd;
      const float v = to_f((prow + v0 + h * vd)[ok ? (unsigned)(tk * (int)ldp + c) : 0u]);
      prev[u] = ok ? v : 0.f;
    }
  };
  auto stash = [&](float* buf, int i0) {
    const int nt = n - i0 < TB ? n - i0 : TB;
#pragma unroll
    for (int u = 0; u < PRE; ++u) {
      if (NT * u >= nt << lr) break;
      const int e = tid + NT * u, tk = e >> lr, row = e & (rows - 1);
      if (tk < nt) {
        float* dst = buf + (tk * R + row / DL_DR) * DL_SEG + row % DL_DR;
#pragma unroll
        for (int a = 0; a < NA; ++a) dst[a * qsz] = pre[a][u];
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (NT * u >= nt << lw) break;
      const int e = tid + NT * u;
      if (e >> lw < nt) buf[NA * qsz + e] = prev[u];
    }
    if (GB && tid < 2 * TB) buf[NA * qsz + TB * wcols + tid] = preg;
  };
  if (n > 0) { fetch(0); stash(smem, 0); }
  __syncthreads();
  int cur = 0;
  for (int i0 = 0; i0 < n; i0 += TB) {
    const bool more = i0 + TB < n;
    if (more) fetch(i0 + TB);
    const float* buf = smem + cur * bufsz;
    const int nt = n - i0 < TB ? n - i0 : TB;
    for (int tk = 0; tk < nt; ++tk) {
      const int seg = (tk * R + r) * DL_SEG;
      const float4* r4 = reinterpret_cast<const float4*>(buf + seg);
      const float4* k4 = reinterpret_cast<const float4*>(buf + KI * qsz + seg);
      const float4* w4 = reinterpret_cast<const float4*>(buf + (NA == 3 ? 2 : 1) * qsz + seg);      // (NA == 5, 3)
      const float4* n4 = NA == 5 ? reinterpret_cast<const float4*>(buf + 2 * qsz + seg) : k4;
      const float4* b4 = reinterpret_cast<const float4*>(buf + (NA == 5 ? 3 * qsz : 0) + seg);   // (NA == 5)
      const float v = buf[NA * qsz + tk * wcols + lc];
      // n . s over the old state (with a decay per channel over the decayed state)
      float acc[4] = {0.f, 0.f, 0.f, 0.f}, dot = 0.f;
      if (MODE != DL_SPACE) {
#pragma unroll
        for (int k = 0; k < DL_DR / 4; ++k) {
          if (MODE == DL_CHANNEL) {
            const float4 w = w4[k];
            S[4 * k] *= w.x; S[4 * k + 1] *= w.y; S[4 * k + 2] *= w.z; S[4 * k + 3] *= w.w;
          }
          const float4 a = n4[k];
          acc[0] += S[4 * k] * a.x; acc[1] += S[4 * k + 1] * a.y; acc[2] += S[4 * k + 2] * a.z; acc[3] += S[4 * k + 3] * a.w;
        }
        dot = group_sum((acc[0] + acc[1]) + (acc[2] + acc[3]), R);
        acc[0] = acc[1] = acc[2] = acc[3] = 0.f;
      }
      if (MODE == DL_CHANNEL && !out) {                      // (only the end states are wanted)
        const float c = buf[NA * qsz + TB * wcols + 2 * tk + 1] * (v - dot);
#pragma unroll
        for (int k = 0; k < DL_DR / 4; ++k) {
          const float4 kk = k4[k];
          S[4 * k] += kk.x * c;
          S[4 * k + 1] += kk.y * c;
          S[4 * k + 2] += kk.z * c;
          S[4 * k + 3] += kk.w * c;
        }
        continue;
      }
      if (MODE == DL_CHANNEL) {
        const float c = buf[NA * qsz + TB * wcols + 2 * tk + 1] * (v - dot);
#pragma unroll
        for (int k = 0; k < DL_DR / 4; ++k) {
          const float4 kk = k4[k], q = r4[k];
          S[4 * k] += kk.x * c;
          S[4 * k + 1] += kk.y * c;
          S[4 * k + 2] += kk.z * c;
          S[4 * k + 3] += kk.w * c;
          acc[0] += S[4 * k] * q.x; acc[1] += S[4 * k + 1] * q.y; acc[2] += S[4 * k + 2] * q.z; acc[3] += S[4 * k + 3] * q.w;
        }
      } else if (GB) {
        const float2 gs = *reinterpret_cast<const float2*>(buf + NA * qsz + TB * wcols + 2 * tk);
        const float w = gs.x, c = MODE == DL_SPACE ? gs.y * v : gs.y * (v - w * dot);
#pragma unroll
        for (int k = 0; k < DL_DR / 4; ++k) {
          const float4 kk = k4[k], q = r4[k];
          S[4 * k] = w * S[4 * k] + kk.x * c;
          S[4 * k + 1] = w * S[4 * k + 1] + kk.y * c;
          S[4 * k + 2] = w * S[4 * k + 2] + kk.z * c;
          S[4 * k + 3] = w * S[4 * k + 3] + kk.w * c;
          acc[0] += S[4 * k] * q.x; acc[1] += S[4 * k + 1] * q.y; acc[2] += S[4 * k + 2] * q.z; acc[3] += S[4 * k + 3] * q.w;
        }
      } else {
#pragma unroll
        for (int k = 0; k < DL_DR / 4; ++k) {
          const float4 w = w4[k], bb = b4[k], kk = k4[k], q = r4[k];
          S[4 * k] = w.x * S[4 * k] - bb.x * dot + kk.x * v;
          S[4 * k + 1] = w.y * S[4 * k + 1] - bb.y * dot + kk.y * v;
          S[4 * k + 2] = w.z * S[4 * k + 2] - bb.z * dot + kk.z * v;
          S[4 * k + 3] = w.w * S[4 * k + 3] - bb.w * dot + kk.w * v;
          acc[0] += S[4 * k] * q.x; acc[1] += S[4 * k + 1] * q.y; acc[2] += S[4 * k + 2] * q.z; acc[3] += S[4 * k + 3] * q.w;
        }
      }
      const float tot = group_sum((acc[0] + acc[1]) + (acc[2] + acc[3]), R) + (MODE == DL_SPACE ? skip * v : 0.f);
      if (out && r == 0 && colok) out[(int64_t)(start + i0 + tk) * (H * vd) + h * vd + col] = tot;
    }
    if (more) stash(smem + (cur ^ 1) * bufsz, i0 + TB);
    __syncthreads();
    cur ^= 1;
  }
#pragma unroll
  for (int k = 0; k < DL_DR; ++k) {
    const int row = row0 + k;
    if (colok && row < d) sp[(unsigned)(row * vd + col)] = S[k];
  }
}

template <int MODE>
static int launch_delta_scan(const float* rf, const float* wf, const float* nf, const float* bf, const float* kf, const float* gb, int G,
                             const void* P, int64_t ldp, int v0, float* state, float* out, int H, int d, int vd, int values, float* trans,
                             SpaceArgs ss, Batch bt, int dtype, hipStream_t st) {
  constexpr int NA = MODE == DL_GENERAL ? 5 : MODE == DL_CHANNEL ? 3 : 2;
  if (bt.B <= 0 || H <= 0 || d <= 0 || vd <= 0 || d > DL_DR * 64 || (values && !P)) return -1;
  if (ldp > 1 << 24 || (int64_t)d * vd > 1 << 30 || (int64_t)H * d > 1 << 24) return -1;         // (offsets inside a block and a state are 32-bit)
  if (trans && (out || !values || bt.B > 32767)) return -1;
  int R = 1;
  while (R * DL_DR < d) R <<= 1;
  const int cols = trans && d > vd ? d : vd;
  const int nw = cols <= 2 * (64 / R) ? 2 : 4;              // wavefronts of a workgroup: no more than the columns ask for
  const int wcols = nw * (64 / R);
  int TB = DL_TBR / R < 16 ? DL_TBR / R : 16;
  if (TB * wcols > 4 * 64 * nw) TB = 4 * 64 * nw / wcols;   // the value look-ahead holds 4 floats per thread
  if (TB < 1) return -1;
  // (2 TB <= 32 threads bring a token's two scalars; TB wcols and a buffer's parts are multiples of 16 bytes)
  const size_t sm = 2 * (size_t)(NA * TB * R * DL_SEG + TB * wcols + (MODE != DL_GENERAL ? (2 * TB + 3) & ~3 : 0)) * sizeof(float);
  const dim3 grid((cols + wcols - 1) / wcols, H, trans ? 2 * bt.B : bt.B);
  RAGGED_DISPATCH(dtype,
    if (nw == 2) hipLaunchKernelGGL((delta_scan_kernel<T, 2, MODE>), grid, dim3(128), sm, st, rf, wf, nf, bf, kf, gb, G, (const T*)P, ldp,
                                    v0, state, out, H, d, vd, trans, R, TB, values, ss, bt);
    else hipLaunchKernelGGL((delta_scan_kernel<T, 4, MODE>), grid, dim3(256), sm, st, rf, wf, nf, bf, kf, gb, G, (const T*)P, ldp, v0,
                            state, out, H, d, vd, trans, R, TB, values, ss, bt))
  return RAGGED_LAUNCH_OK();
}

// out may be null (only the end states are wanted); values = 0: the value columns of P are not read and count as 0; trans (with
// values, without out): the chunks' transition matrices in the same launch
extern "C" int ragged_delta_scan(const float* rf, const float* wf, const float* nf, const float* bf, const float* kf, const void* P,
                                 int64_t ldp, int v0, float* state, float* out, int H, int d, int vd, int values, float* trans, Batch bt,
                                 int dtype, hipStream_t st) {
  return launch_delta_scan<DL_GENERAL>(rf, wf, nf, bf, kf, nullptr, H, P, ldp, v0, state, out, H, d, vd, values, trans, SpaceArgs{}, bt, dtype, st);
}

// the gated rule: qf, kf [rows, G d], gb [rows, H, 2]; wf [rows, H d] or null: a decay per key channel
extern "C" int ragged_gated_delta_scan(const float* qf, const float* kf, const float* wf, const float* gb, int G, const void* P, int64_t ldp, int v0,
                                       float* state, float* out, int H, int d, int vd, int values, float* trans, Batch bt, int dtype, hipStream_t st) {
  if (G <= 0 || H % G || !gb) return -1;
  if (wf) return launch_delta_scan<DL_CHANNEL>(qf, wf, nullptr, nullptr, kf, gb, G, P, ldp, v0, state, out, H, d, vd, values, trans, SpaceArgs{}, bt,
                                               dtype, st);
  return launch_delta_scan<DL_GATED>(qf, nullptr, nullptr, nullptr, kf, gb, G, P, ldp, v0, state, out, H, d, vd, values, trans, SpaceArgs{}, bt, dtype, st);
}

// the state space recurrence: X [rows, ldx] of type T holds x (columns 0 .. H vd), B and C (columns b0 .., c0 .., G d each)
extern "C" int ragged_state_space_scan(SpaceArgs ss, const void* X, int64_t ldx, int G, float* state, float* out, int H, int d, int vd,
                                       Batch bt, int dtype, hipStream_t st) {
  if (G <= 0 || H % G || !ss.dt || !ss.dt_bias || !ss.rate || !ss.D || ss.lddt < H || ss.b0 < 0 || ss.c0 < 0) return -1;
  if (ldx < (int64_t)H * vd || ldx < ss.b0 + (int64_t)G * d || ldx < ss.c0 + (int64_t)G * d || !out) return -1;
  return launch_delta_scan<DL_SPACE>(nullptr, nullptr, nullptr, nullptr, nullptr, nullptr, G, X, ldx, 0, state, out, H, d, vd, 1, nullptr, ss, bt, dtype, st);
}

// ---------------------------------------------------------------------------------------------------------------
// Long portions are cut into chunks that are scanned side by side.  A chunk maps the state at its start linearly,
// S_end = A_c S_start + L_c (A_c [d, d] per head: the chunk scanned without inputs from the identity; L_c: the chunk
// scanned from zero).  This kernel walks a sequence's chunks one after the other: begin[c] <- S, S <- A_c S + L_c, and
// leaves the last S in the sequence's slot.  A workgroup holds 16 columns of S in LDS; thread (i0, j) makes rows
// i0, i0 + 16, ... of column j.  Grid: (column blocks, heads, sequences); cfirst[b] .. cfirst[b + 1] - 1 are b's chunks.
constexpr int DC_COLS = 16;
constexpr int DC_LDS_D = 128;                              // up to this many rows a chunk's A is staged in LDS

// NU > 0: a thread makes rows i0 + 16 u, u < NU (16 NU >= d).  A_c is brought into LDS by the whole workgroup (coalesced) and
// A_c and the thread's elements of L_c are requested one chunk ahead into registers, so a chunk's step waits for no memory;
// S lies transposed, [column][row], so that both operands are read four channels at a time.
// NU = 0: any d; every thread reads its rows of A_c and its elements of L_c from memory as it goes.
template <int NU>
__global__ __launch_bounds__(256) void delta_chain_kernel(float* __restrict__ state, const float* __restrict__ local,
                                                          const float* __restrict__ trans, float* __restrict__ begin,
                                                          const int* __restrict__ cfirst, const int* __restrict__ seq_past,
                                                          const int* __restrict__ seq_slot, int H, int d, int vd) {
  extern __shared__ __attribute__((aligned(16))) float smem[];   // two buffers [DC_COLS][ld] of S, then A [d][ld]
  constexpr int U = NU > 0 ? NU : 1, NA = NU * NU > 0 ? NU * NU : 1;      // d d <= 256 NU NU
  const int b = blockIdx.z, h = blockIdx.y;
  const int j = threadIdx.x % DC_COLS, i0 = threadIdx.x / DC_COLS, col = blockIdx.x * DC_COLS + j;
  const bool colok = col < vd;
  const int cc = colok ? col : vd - 1;
  const int ld = ((d + 3) & ~3) + 4;                         // (a row's padding stays zero; the odd multiple of 4 spreads the banks)
  float* cur = smem;
  float* nxt = smem + DC_COLS * ld;
  float* As = smem + 2 * DC_COLS * ld;
  float* sp = state + ((int64_t)seq_slot[b] * H + h) * d * vd;
  const bool old = seq_past[b] > 0;
  for (int e = threadIdx.x; e < (2 * DC_COLS + (NU > 0 ? d : 0)) * ld; e += 256) smem[e] = 0.f;
  __syncthreads();
  for (int i = i0; i < d; i += 16) cur[j * ld + i] = old ? sp[(int64_t)i * vd + cc] : 0.f;
  const int c0 = cfirst[b], c1 = cfirst[b + 1];
  float apre[NA], lpre[U], acc[U];
  auto fetch = [&](int c) {
    const float* A = trans + ((int64_t)c * H + h) * d * d;
    const float* L = local + ((int64_t)c * H + h) * d * vd;
#pragma unroll
    for (int u = 0; u < NA; ++u) {
      const int e = threadIdx.x + 256 * u;
      apre[u] = A[e < d * d ? e : d * d - 1];
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int i = i0 + 16 * u;
      lpre[u] = L[(int64_t)(i < d ? i : d - 1) * vd + cc];
    }
  };
  const int step_r = 256 / d, step_c = 256 % d;
  if (NU > 0 && c0 < c1) fetch(c0);
  __syncthreads();
  for (int c = c0; c < c1; ++c) {
    float* B = begin + ((int64_t)c * H + h) * d * vd;
    if (NU > 0) {
      int ar = threadIdx.x / d, ac = threadIdx.x % d;        // element e = threadIdx.x + 256 u of A sits at (e / d, e % d)
#pragma unroll
      for (int u = 0; u < NA; ++u) {
        if (ar < d) As[ar * ld + ac] = apre[u];
        ar += step_r;
        ac += step_c;
        if (ac >= d) { ac -= d; ++ar; }
      }
#pragma unroll
      for (int u = 0; u < U; ++u) acc[u] = lpre[u];
      __syncthreads();
      if (c + 1 < c1) fetch(c + 1);
      for (int l = 0; l < d; l += 4) {
        const float4 s = *reinterpret_cast<const float4*>(cur + j * ld + l);
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const int i = i0 + 16 * u;
          const float4 a = *reinterpret_cast<const float4*>(As + (i < d ? i : d - 1) * ld + l);
          acc[u] += (a.x * s.x + a.y * s.y) + (a.z * s.z + a.w * s.w);
        }
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int i = i0 + 16 * u;
        if (i < d) {
          if (colok) B[(int64_t)i * vd + col] = cur[j * ld + i];
          nxt[j * ld + i] = acc[u];
        }
      }
    } else {
      const float* A = trans + ((int64_t)c * H + h) * d * d;
      const float* L = local + ((int64_t)c * H + h) * d * vd;
      for (int i = i0; i < d; i += 16) {
        if (colok) B[(int64_t)i * vd + col] = cur[j * ld + i];
        float s4[4] = {L[(int64_t)i * vd + cc], 0.f, 0.f, 0.f};
        const float* ar = A + (int64_t)i * d;
        int l = 0;
        for (; l + 4 <= d; l += 4) {
#pragma unroll
          for (int k = 0; k < 4; ++k) s4[k] += ar[l + k] * cur[j * ld + l + k];
        }
        for (; l < d; ++l) s4[0] += ar[l] * cur[j * ld + l];
        nxt[j * ld + i] = (s4[0] + s4[1]) + (s4[2] + s4[3]);
      }
    }
    __syncthreads();
    float* t = cur; cur = nxt; nxt = t;
  }
  for (int i = i0; i < d; i += 16)
    if (colok) sp[(int64_t)i * vd + col] = cur[j * ld + i];
}

extern "C" int ragged_delta_chain_ok(int d) { return d > 0 && d <= 384; }

template <int NU>
static int launch_delta_chain(float* state, const float* local, const float* trans, float* begin, const int* cfirst, const int* seq_past,
                              const int* seq_slot, int B, int H, int d, int vd, hipStream_t st) {
  const size_t ld = ((d + 3) & ~3) + 4, sm = (2 * DC_COLS + (NU > 0 ? d : 0)) * ld * sizeof(float);
  if (sm > 64 * 1024) {                                      // (asked for once per process and kernel)
    static const hipError_t asked = hipFuncSetAttribute(reinterpret_cast<const void*>(delta_chain_kernel<NU>),
                                                        hipFuncAttributeMaxDynamicSharedMemorySize, 96 * 1024);
    if (asked != hipSuccess) return -3;
  }
  hipLaunchKernelGGL(delta_chain_kernel<NU>, dim3((vd + DC_COLS - 1) / DC_COLS, H, B), dim3(256), sm, st, state, local, trans, begin, cfirst,
                     seq_past, seq_slot, H, d, vd);
  return RAGGED_LAUNCH_OK();
}

extern "C" int ragged_delta_chain(float* state, const float* local, const float* trans, float* begin, const int* cfirst,
                                  const int* seq_past, const int* seq_slot, int B, int H, int d, int vd, hipStream_t st) {
  if (B <= 0 || H <= 0 || vd <= 0 || !ragged_delta_chain_ok(d)) return -1;
#define DC_CASE(NU) return launch_delta_chain<NU>(state, local, trans, begin, cfirst, seq_past, seq_slot, B, H, d, vd, st)
  if (d <= 16) DC_CASE(1);
  if (d <= 32) DC_CASE(2);
  if (d <= 48) DC_CASE(3);
  if (d <= 64) DC_CASE(4);
  if (d <= 96) DC_CASE(6);
  if (d <= DC_LDS_D) DC_CASE(8);
  DC_CASE(0);
#undef DC_CASE
}
