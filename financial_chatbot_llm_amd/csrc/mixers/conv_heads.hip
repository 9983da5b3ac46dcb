// Short causal convolution of projected query, key and value heads, with what follows it up to attention:
//
//   y_t[c] = sum_j w[c][j] * u_(t - (K-1) + j)[c]      per channel, zeros before the sequence's start, no activation
//   q, k:  y / sqrt(mean(y^2) + eps) * weight[D]       per head, the weight shared by the heads (null: no norm)
//   q:     times 1 + coef * ln(floor((p + 1) / every) + 1) at position p (coef 0: none)  -> qout [T, H*D]
//   k, v:  -> cache row slots[t] of [k: G*D | v: G*P]
//
// over a flat batch of segments (prompt chunks and single decoded tokens alike).  Segment s keeps its last K-1
// projected inputs in slot slot[s] of `state` (f32 [slots, K-1, C]); a segment that starts at position 0 starts from
// zeros whatever the slot held.  G = 0: queries only (a layer that reads another layer's keys and values).
//
// A wave owns one head and TT consecutive rows of a segment: all TT + K - 1 input rows are fetched before the first
// is used (the loads overlap), the convolution runs from registers and each row's norm is one wave reduction.
// Only the wave of a segment's first tile reads the slot's history (TT >= K - 1), and it is the one that replaces it.
#include "mx_common.h"

namespace {

constexpr int CH_WAVES = 4;

// VE adjacent channels per lane and access, NC accesses per row, up to KM taps
template <typename T, int VE, int NC, int KM, int TT>
__global__ void __launch_bounds__(CH_WAVES * 64)
conv_heads_kernel(const T* __restrict__ in, long si, const float* __restrict__ w, int K, float* state,
                  const float* __restrict__ qw, const float* __restrict__ kw, float eps, float tcoef, int tevery,
                  const int* __restrict__ cu, const int* __restrict__ slot, const int* __restrict__ pos,
                  const int* __restrict__ slots, T* __restrict__ cache, T* __restrict__ qout, int H, int G, int D, int P) {
  static_assert(TT >= KM - 1, "tiles behind the first must not reach the slot's history");
  typedef T vt __attribute__((ext_vector_type(VE)));
  constexpr int NV = NC * VE;
  const int s = blockIdx.z;
  const int r0 = cu[s], n = cu[s + 1] - r0;
  const int t0 = blockIdx.x * TT;
  const int unit = blockIdx.y * CH_WAVES + (threadIdx.x >> 6);
  if (t0 >= n || unit >= H + 2 * G) return;              // wave-uniform, no block barrier below
  const int lane = threadIdx.x & 63;
  const bool isq = unit < H, isv = unit >= H + G;
  const int nd = isv ? P : D;
  const int col = isq ? unit * D : (isv ? (H + G) * D + (unit - H - G) * P : unit * D);   // channels are q | k | v
  const int C = (H + G) * D + G * P;
  const int sl = slot[s];
  const bool fresh = sl < 0 || pos[r0] == 0;
  float* st = state + (sl < 0 ? 0 : (long)sl * (K - 1) * C) + col;
  const int pad = KM - K;                                // taps are aligned to the end of the KM-wide window

  float x[TT + KM - 1][NV], wk[KM][NV];
#pragma unroll
  for (int r = 0; r < TT + KM - 1; ++r) {
    const int j = t0 - (KM - 1) + r;                     // row of the segment, < 0: history
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int d = (c * 64 + lane) * VE;
#pragma unroll
      for (int e = 0; e < VE; ++e) x[r][c * VE + e] = 0.f;
      if (d < nd) {
        if (j >= 0) {
          if (j < n) {
            const vt v = *reinterpret_cast<const vt*>(in + (long)(r0 + j) * si + col + d);
#pragma unroll
            for (int e = 0; e < VE; ++e) x[r][c * VE + e] = (float)v[e];
          }
        } else if (!fresh && K - 1 + j >= 0) {
#pragma unroll
          for (int e = 0; e < VE; ++e) x[r][c * VE + e] = st[(long)(K - 1 + j) * C + d + e];
        }
      }
    }
  }
#pragma unroll
  for (int k = 0; k < KM; ++k)
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int e = 0; e < VE; ++e) {
        const int d = (c * 64 + lane) * VE + e;
        wk[k][c * VE + e] = (d < nd && k >= pad) ? w[(long)(col + d) * K + k - pad] : 0.f;
      }
  // the slot's next history: entry e is the input K-1-e rows before the segment's end (entries move down, so each
  // is read before it is overwritten; a lane touches its own channels only)
  if (t0 == 0 && sl >= 0) {
    for (int e = 0; e < K - 1; ++e) {
      const int i = n - (K - 1) + e;
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        const int d = (c * 64 + lane) * VE;
        if (d < nd) {
#pragma unroll
          for (int q = 0; q < VE; ++q)
            st[(long)e * C + d + q] = i >= 0 ? ldf(in + (long)(r0 + i) * si + col + d + q)
                                             : (fresh ? 0.f : st[(long)(e + n) * C + d + q]);
        }
      }
    }
  }
  float nw[NV];
  const float* wn = isq ? qw : (isv ? nullptr : kw);
  if (wn != nullptr)
#pragma unroll
    for (int c = 0; c < NC; ++c)
#pragma unroll
      for (int e = 0; e < VE; ++e) {
        const int d = (c * 64 + lane) * VE + e;
        nw[c * VE + e] = d < nd ? wn[d] : 0.f;
      }
  const int Wr = G * (D + P);
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    if (t0 + i >= n) break;
    const long row = r0 + t0 + i;
    float y[NV], ss = 0.f;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      float a = 0.f;
#pragma unroll
      for (int k = 0; k < KM; ++k) a += wk[k][v] * x[i + k][v];
      y[v] = a;
      ss += a * a;
    }
    if (wn != nullptr) {
      const float f = 1.0f / sqrtf(mx_wave_sum(ss) / (float)nd + eps);
#pragma unroll
      for (int v = 0; v < NV; ++v) y[v] *= f * nw[v];
    }
    T* dst;
    if (isq) {
      if (tcoef != 0.f) {
        const float f = 1.0f + tcoef * logf((float)((pos[row] + 1) / tevery + 1));
#pragma unroll
        for (int v = 0; v < NV; ++v) y[v] *= f;
      }
      dst = qout + row * (long)H * D + (long)unit * D;
    } else {
      const int cr = slots[row];
      if (cr < 0) continue;
      dst = cache + (long)cr * Wr + (isv ? G * D + (unit - H - G) * P : (unit - H) * D);
    }
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      const int d = (c * 64 + lane) * VE;
      if (d < nd) {
        vt o;
#pragma unroll
        for (int e = 0; e < VE; ++e) o[e] = (T)y[c * VE + e];
        *reinterpret_cast<vt*>(dst + d) = o;
      }
    }
  }
}

}  // namespace

// in: [T, C] slice (row stride si) of storage type dt, channels q: H*D | k: G*D | v: G*P; w f32 [C, K] (last column:
// the current token's tap), 1 <= K <= 16; state f32 [slots, K-1, C] (unused for K = 1); qw / kw f32 [D] or null;
// cu [S+1] row bounds, slot [S] (< 0: no history kept), pos [T], slots [T] cache rows (< 0: no write);
// cache [rows, G*(D+P)] (unused for G = 0) and qout [T, H*D] of storage type dt
MX_API int mx_conv_heads(const void* in, long si, int dt, const float* w, int K, float* state, const float* qw,
                         const float* kw, float eps, float tcoef, int tevery, const int* cu, const int* slot,
                         const int* pos, const int* slots, void* cache, void* qout, int S, int max_len, int H, int G,
                         int D, int P, hipStream_t st) {
  if (S <= 0 || max_len <= 0) return 0;
  const int big = G > 0 && P > D ? P : D;
  if (K < 1 || K > 16 || H < 1 || G < 0 || D < 1 || P < 1 || big > 512 || tevery < 1 || (K > 1 && state == nullptr) ||
      (G > 0 && cache == nullptr))
    return (int)hipErrorInvalidValue;
  const size_t al = dt == 1 ? 8 : 4;                       // two elements
  const bool two = D % 2 == 0 && (G == 0 || P % 2 == 0) && si % 2 == 0 && ((size_t)in | (size_t)qout | (size_t)cache) % al == 0;
  const int units = H + 2 * G;
#define CH_LAUNCH(VE, NC, KM, TT)                                                                                     \
  do {                                                                                                                \
    dim3 grid((max_len + TT - 1) / TT, (units + CH_WAVES - 1) / CH_WAVES, S);                                         \
    MX_DISPATCH(dt, TY, conv_heads_kernel<TY, VE, NC, KM, TT><<<grid, CH_WAVES * 64, 0, st>>>(                        \
        (const TY*)in, si, w, K, state, qw, kw, eps, tcoef, tevery, cu, slot, pos, slots, (TY*)cache, (TY*)qout, H, G, \
        D, P));                                                                                                       \
  } while (0)
#define CH_TAPS(VE, NC)                     \
  do {                                      \
    if (K <= 4) CH_LAUNCH(VE, NC, 4, 8);    \
    else if (K <= 8) CH_LAUNCH(VE, NC, 8, 8); \
    else CH_LAUNCH(VE, NC, 16, 16);         \
  } while (0)
  if (two) {
    if (big <= 128) CH_TAPS(2, 1);
    else if (big <= 256) CH_TAPS(2, 2);
    else CH_TAPS(2, 4);
  } else {
    if (big <= 128) CH_TAPS(1, 2);
    else CH_TAPS(1, 8);
  }
#undef CH_TAPS
#undef CH_LAUNCH
  MX_RETURN_LAUNCH();
}
