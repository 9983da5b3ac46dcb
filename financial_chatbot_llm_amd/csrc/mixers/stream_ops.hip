// The 32-bit residual stream and the small per-row passes around it:
//   * embedding gather into an f32 stream;
//   * parallel-block residual update fused with the next RMS norm:
//         x <- x + mult * (a + b);  y = x / sqrt(mean(x^2) + eps) * w
//     optionally with a weight per sublayer output and a sigmoid gate per element on the update:
//         x <- x + sigmoid(gate + gate_bias) * (mult_a * a + mult_b * b)
//     and with a token's embedding row added after the update, or the stream starting from it;
//   * RMS norm of a strided row slice (latent norms), optionally in equal groups and with a SiLU
//     gate applied first (the state-space mixer's output norm);
//   * elementwise norms D(v) = tanh(alpha v) * w + b around a sublayer, one pass over the stream:
//         x <- x + D1(y) (or x <- D1(scale * table[id]) at the embedding);  out = D2(x)
//   * activations: relu^2, and the clamped gated unit g * sigmoid(alpha g) * (u + 1);
//   * biased top-k routing: softmax or sigmoid scores, choice = score + bias, weights = unbiased scores,
//     optionally divided by the sum of the chosen ones and times a constant;
//   * weighted combine of routed expert rows, identity experts and a shared expert.
#include "mx_common.h"

namespace {

template <typename T>
__global__ void embed_kernel(const int* __restrict__ ids, const T* __restrict__ table, float* __restrict__ out,
                             int W, int V) {
  const int t = blockIdx.x;
  int id = ids[t];
  id = id < 0 ? 0 : (id >= V ? V - 1 : id);
  const T* row = table + (long)id * W;
  for (int i = threadIdx.x; i < W; i += blockDim.x) out[(long)t * W + i] = ldf(row + i);
}

// one block per row.  a / b: the two sublayer outputs of a parallel block (either may be null);
// gate (may be null): pre-activations of a sigmoid gate on the update, gate_bias f32 [W] or null;
// table (may be null): row ids[t] of [vocab, W] is added after the update or, fresh, replaces x.
template <typename TA, typename TO>
__global__ void residual_norm_kernel(float* __restrict__ x, const TA* __restrict__ a, long sa,
                                     const TA* __restrict__ b, long sb, float mult, float mult_b,
                                     const TA* __restrict__ gate, long sg, const float* __restrict__ gate_bias,
                                     const int* __restrict__ ids, const TA* __restrict__ table, int vocab, int fresh,
                                     const float* __restrict__ w, float eps, TO* __restrict__ out, int W) {
  __shared__ float scratch[16];
  const long t = blockIdx.x;
  float* xr = x + t * W;
  const TA* er = table != nullptr ? table + (long)min(max(ids[t], 0), vocab - 1) * W : nullptr;
  float ss = 0.f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    float v = fresh ? 0.f : xr[i];
    if (a != nullptr || b != nullptr) {
      float s;
      if (mult == mult_b) {
        s = 0.f;
        if (a != nullptr) s += ldf(a + t * sa + i);
        if (b != nullptr) s += ldf(b + t * sb + i);
        s *= mult;
      } else {
        s = (a != nullptr ? mult * ldf(a + t * sa + i) : 0.f) + (b != nullptr ? mult_b * ldf(b + t * sb + i) : 0.f);
      }
      if (gate != nullptr) s *= mx_sigmoid(ldf(gate + t * sg + i) + (gate_bias != nullptr ? gate_bias[i] : 0.f));
      v = v + s;
    }
    if (er != nullptr) v += ldf(er + i);
    if (a != nullptr || b != nullptr || er != nullptr) xr[i] = v;
    ss += v * v;
  }
  if (out == nullptr) return;
  ss = mx_block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x) stf(out + t * W + i, xr[i] * r * w[i]);
}

// the same with four adjacent columns per access and the row in registers between its two passes: a thread owns NC
// groups of columns; every row start and W are multiples of four elements
template <typename TA, typename TO, int NC>
__global__ void residual_norm_vec_kernel(float* __restrict__ x, const TA* __restrict__ a, long sa,
                                         const TA* __restrict__ b, long sb, float mult, float mult_b,
                                         const TA* __restrict__ gate, long sg, const float* __restrict__ gate_bias,
                                         const int* __restrict__ ids, const TA* __restrict__ table, int vocab, int fresh,
                                         const float* __restrict__ w, float eps, TO* __restrict__ out, int W) {
  typedef float vf __attribute__((ext_vector_type(4)));
  typedef TA va __attribute__((ext_vector_type(4)));
  typedef TO vo __attribute__((ext_vector_type(4)));
  __shared__ float scratch[16];
  const long t = blockIdx.x;
  float* xr = x + t * W;
  const TA* er = table != nullptr ? table + (long)min(max(ids[t], 0), vocab - 1) * W : nullptr;
  const bool upd = a != nullptr || b != nullptr;
  vf v[NC];
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = (threadIdx.x + c * blockDim.x) * 4;
    v[c] = vf{0.f, 0.f, 0.f, 0.f};
    if (i >= W) continue;
    if (!fresh) v[c] = *reinterpret_cast<const vf*>(xr + i);
    if (upd) {
      va av = va{}, bv = va{};
      if (a != nullptr) av = *reinterpret_cast<const va*>(a + t * sa + i);
      if (b != nullptr) bv = *reinterpret_cast<const va*>(b + t * sb + i);
      vf s;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        s[e] = mult == mult_b ? mult * ((float)av[e] + (float)bv[e]) : mult * (float)av[e] + mult_b * (float)bv[e];
      if (gate != nullptr) {
        const va gv = *reinterpret_cast<const va*>(gate + t * sg + i);
#pragma unroll
        for (int e = 0; e < 4; ++e) s[e] *= mx_sigmoid((float)gv[e] + (gate_bias != nullptr ? gate_bias[i + e] : 0.f));
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) v[c][e] += s[e];
    }
    if (er != nullptr) {
      const va ev = *reinterpret_cast<const va*>(er + i);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[c][e] += (float)ev[e];
    }
    if (upd || er != nullptr) *reinterpret_cast<vf*>(xr + i) = v[c];
#pragma unroll
    for (int e = 0; e < 4; ++e) ss += v[c][e] * v[c][e];
  }
  if (out == nullptr) return;
  ss = mx_block_sum(ss, scratch);
  const float r = 1.0f / sqrtf(ss / (float)W + eps);
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int i = (threadIdx.x + c * blockDim.x) * 4;
    if (i >= W) continue;
    const vf wv = *reinterpret_cast<const vf*>(w + i);
    vo o;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] = (TO)(v[c][e] * r * wv[e]);
    *reinterpret_cast<vo*>(out + t * W + i) = o;
  }
}

// grid (rows, groups): RMS norm of `n` contiguous elements per group.  gate (optional): the
// element is multiplied by silu(gate) BEFORE the statistics.
template <typename TI, typename TG, typename TO>
__global__ void group_norm_kernel(const TI* __restrict__ in, long si, const TG* __restrict__ gate, long sg,
                                  const float* __restrict__ w, float eps, TO* __restrict__ out, long so, int n) {
  __shared__ float scratch[16];
  const long t = blockIdx.x;
  const int g = blockIdx.y;
  const TI* r = in + t * si + (long)g * n;
  const TG* z = gate == nullptr ? nullptr : gate + t * sg + (long)g * n;
  float ss = 0.f;
  for (int i = threadIdx.x; i < n; i += blockDim.x) {
    float v = ldf(r + i);
    if (z != nullptr) v *= mx_silu(ldf(z + i));
    ss += v * v;
  }
  ss = mx_block_sum(ss, scratch);
  const float k = 1.0f / sqrtf(ss / (float)n + eps);
  for (int i = threadIdx.x; i < n; i += blockDim.x) {
    float v = ldf(r + i);
    if (z != nullptr) v *= mx_silu(ldf(z + i));
    stf(out + t * so + (long)g * n + i, v * k * w[(long)g * n + i]);
  }
}

template <typename T>
__global__ void relu2_kernel(const T* __restrict__ in, long si, T* __restrict__ out, long so, int n, long total) {
  for (long i = blockIdx.x * (long)blockDim.x + threadIdx.x; i < total; i += (long)gridDim.x * blockDim.x) {
    const long t = i / n;
    const int c = (int)(i - t * n);
    const float v = fmaxf(ldf(in + t * si + c), 0.f);
    stf(out + t * so + c, v * v);
  }
}

// grid (row groups, column chunks): a thread owns V adjacent columns and walks `rows` rows, its weights in
// registers.  a null: the first form reads table rows (ids) and REPLACES x; both a and table null: out only.
template <typename TA, typename TO, int V>
__global__ void dyn_tanh_kernel(float* __restrict__ x, const TA* __restrict__ a, long sa, const int* __restrict__ ids,
                                const TA* __restrict__ table, int vocab, float scale, float alpha1,
                                const float* __restrict__ w1, const float* __restrict__ b1, float alpha2,
                                const float* __restrict__ w2, const float* __restrict__ b2, TO* __restrict__ out, int W,
                                int rows, int T) {
  typedef float vf __attribute__((ext_vector_type(V)));
  typedef TA va __attribute__((ext_vector_type(V)));
  typedef TO vo __attribute__((ext_vector_type(V)));
  const int c = (blockIdx.y * blockDim.x + threadIdx.x) * V;
  if (c >= W) return;
  const bool pre = a != nullptr || table != nullptr;
  vf w1r = {}, b1r = {}, w2r = {}, b2r = {};
  if (pre) {
    w1r = *reinterpret_cast<const vf*>(w1 + c);
    b1r = *reinterpret_cast<const vf*>(b1 + c);
  }
  if (out != nullptr) {
    w2r = *reinterpret_cast<const vf*>(w2 + c);
    b2r = *reinterpret_cast<const vf*>(b2 + c);
  }
  const long t0 = (long)blockIdx.x * rows, t1 = min(t0 + rows, (long)T);
  for (long t = t0; t < t1; ++t) {
    float* xr = x + t * W + c;
    vf v = {};
    if (a != nullptr) {
      const va y = *reinterpret_cast<const va*>(a + t * sa + c);
      v = *reinterpret_cast<const vf*>(xr);
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] += mx_tanh(alpha1 * (float)y[e]) * w1r[e] + b1r[e];
    } else if (table != nullptr) {
      int id = ids[t];
      id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
      const va y = *reinterpret_cast<const va*>(table + (long)id * W + c);
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = mx_tanh(alpha1 * (scale * (float)y[e])) * w1r[e] + b1r[e];
    } else {
      v = *reinterpret_cast<const vf*>(xr);
    }
    if (pre) *reinterpret_cast<vf*>(xr) = v;
    if (out != nullptr) {
      vo o;
#pragma unroll
      for (int e = 0; e < V; ++e) o[e] = (TO)(mx_tanh(alpha2 * v[e]) * w2r[e] + b2r[e]);
      *reinterpret_cast<vo*>(out + t * W + c) = o;
    }
  }
}

// gate and up are column slices (row strides sg / su) of one projection output
template <typename T>
__global__ void glu_clamp_kernel(const T* __restrict__ gate, long sg, const T* __restrict__ up, long su,
                                 float limit, float alpha, T* __restrict__ out, long so, int n, long total) {
  for (long i = blockIdx.x * (long)blockDim.x + threadIdx.x; i < total; i += (long)gridDim.x * blockDim.x) {
    const long t = i / n;
    const int c = (int)(i - t * n);
    const float g = fminf(ldf(gate + t * sg + c), limit);
    const float u = fminf(fmaxf(ldf(up + t * su + c), -limit), limit);
    stf(out + t * so + c, g * mx_sigmoid(alpha * g) * (u + 1.0f));
  }
}

// the same with 16-byte accesses: grid (rows, column chunks), V elements per thread; every row start and the
// column count are multiples of V elements
template <typename T, int V>
__global__ void glu_clamp_vec_kernel(const T* __restrict__ gate, long sg, const T* __restrict__ up, long su, float limit,
                                     float alpha, T* __restrict__ out, long so, int nv) {
  typedef T vec __attribute__((ext_vector_type(V)));
  const long t = blockIdx.x;
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= nv) return;
  const vec gv = *reinterpret_cast<const vec*>(gate + t * sg + (long)c * V);
  const vec uv = *reinterpret_cast<const vec*>(up + t * su + (long)c * V);
  vec o;
#pragma unroll
  for (int e = 0; e < V; ++e) {
    const float g = fminf((float)gv[e], limit);
    const float u = fminf(fmaxf((float)uv[e], -limit), limit);
    o[e] = (T)(g * mx_sigmoid(alpha * g) * (u + 1.0f));
  }
  *reinterpret_cast<vec*>(out + t * so + (long)c * V) = o;
}

// one wave per token: scores = softmax(z) over all E entries, or (sigm) sigmoid(z) of each; the `top` largest
// score + bias are chosen (ties: the lower index), each with its unbiased score as weight -- with renorm divided
// by the chosen scores' sum (+ 1e-20) -- times wscale.
__global__ void route_biased_kernel(const float* __restrict__ z, const float* __restrict__ bias, int E, int top, int sigm,
                                    int renorm, float wscale, float* __restrict__ outw, int* __restrict__ outi, int T) {
  const int t = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (t >= T) return;
  const float* zr = z + (long)t * E;
  float m = -INFINITY, inv = 1.f;
  if (!sigm) {
    for (int e = lane; e < E; e += 64) m = fmaxf(m, zr[e]);
    m = mx_wave_max(m);
    float s = 0.f;
    for (int e = lane; e < E; e += 64) s += expf(zr[e] - m);
    inv = 1.0f / mx_wave_sum(s);
  }
  float wsum = 0.f;                                  // lane 0: the chosen scores' sum
  unsigned long long taken_lo = 0, taken_hi = 0;     // this lane's entries already chosen (E <= 64 * 128)
  for (int k = 0; k < top; ++k) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int e = lane, j = 0; e < E; e += 64, ++j) {
      const bool used = j < 64 ? (taken_lo >> j) & 1 : (taken_hi >> (j - 64)) & 1;
      if (used) continue;
      const float c = (sigm ? mx_sigmoid(zr[e]) : expf(zr[e] - m) * inv) + (bias != nullptr ? bias[e] : 0.f);
      if (c > bv || (c == bv && e < bi)) {
        bv = c;
        bi = e;
      }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ov > bv || (ov == bv && oi < bi)) {
        bv = ov;
        bi = oi;
      }
    }
    if (bi != 0x7fffffff && (bi & 63) == lane) {
      const int j = bi >> 6;
      if (j < 64) taken_lo |= 1ull << j; else taken_hi |= 1ull << (j - 64);
    }
    if (lane == 0) {
      const int e = bi == 0x7fffffff ? 0 : bi;
      outi[(long)t * top + k] = e;
      const float sc = bi == 0x7fffffff ? 0.f : (sigm ? mx_sigmoid(zr[e]) : expf(zr[e] - m) * inv);
      wsum += sc;
      outw[(long)t * top + k] = renorm ? sc : sc * wscale;
    }
  }
  if (renorm && lane == 0) {
    const float f = wscale / (wsum + 1e-20f);
    for (int k = 0; k < top; ++k) outw[(long)t * top + k] *= f;
  }
}

// out[t] = sum_k w[t,k] * src(t,k) (+ shared[t]):  src is the token's own input row h[t] for an
// identity expert (index >= E), else row pos[t,k] of the expert-sorted outputs ys.
template <typename T>
__global__ void moe_combine_kernel(const T* __restrict__ ys, const int* __restrict__ pos, const int* __restrict__ idx,
                                   const float* __restrict__ wts, const T* __restrict__ h, long sh,
                                   const T* __restrict__ shared, long ssh, int E, int top, int W,
                                   T* __restrict__ out) {
  const long t = blockIdx.x;
  for (int c = threadIdx.x; c < W; c += blockDim.x) {
    float acc = shared != nullptr ? ldf(shared + t * ssh + c) : 0.f;
    for (int k = 0; k < top; ++k) {
      const int e = idx[t * top + k];
      const float w = wts[t * top + k];
      if (w == 0.f) continue;
      const float v = e >= E ? ldf(h + t * sh + c) : ldf(ys + (long)pos[t * top + k] * W + c);
      acc += w * v;
    }
    stf(out + t * W + c, acc);
  }
}

}  // namespace

MX_API int mx_embed(const int* ids, const void* table, int dt, float* out, int T, int W, int V, hipStream_t st) {
  if (T <= 0) return 0;
  MX_DISPATCH(dt, TT, embed_kernel<TT><<<T, 256, 0, st>>>(ids, (const TT*)table, out, W, V));
  MX_RETURN_LAUNCH();
}

// x [T, W] f32 (updated in place when a or b is given); out (may be null: update only) of type dt_out;
// a, b, gate (a [T, >= W] slice, or null) and table of type dt_ab; mult weighs a, mult_b weighs b; with a table
// [vocab, W] the row of ids[t] is added after the update or, fresh != 0, x starts from it (its old values unread)
MX_API int mx_residual_norm(float* x, const void* a, long sa, const void* b, long sb, int dt_ab, float mult,
                            float mult_b, const void* gate, long sg, const float* gate_bias, const int* ids,
                            const void* table, int vocab, int fresh, const float* w, float eps, void* out, int dt_out,
                            int T, int W, hipStream_t st) {
  if (T <= 0) return 0;
  if ((table != nullptr && (ids == nullptr || vocab < 1)) || (fresh && table == nullptr) ||
      (out != nullptr && w == nullptr))
    return (int)hipErrorInvalidValue;
  const size_t row = dt_ab == 1 ? 16 : 8;
  const bool vec = W % 4 == 0 && W <= 8192 && sa % 4 == 0 && sb % 4 == 0 && sg % 4 == 0 &&
                   ((size_t)a | (size_t)b | (size_t)gate | (size_t)table) % row == 0 && ((size_t)x | (size_t)w) % 16 == 0 &&
                   (size_t)out % (dt_out == 1 ? 16 : 8) == 0;
  if (vec) {
    const int cols = W / 4, ntv = cols >= 512 ? 512 : (cols + 63) / 64 * 64;
#define RESIDUAL_VEC(NC)                                                                                              \
  MX_DISPATCH(dt_ab, TA, MX_DISPATCH(dt_out, TO, residual_norm_vec_kernel<TA, TO, NC><<<T, ntv, 0, st>>>(             \
      x, (const TA*)a, sa, (const TA*)b, sb, mult, mult_b, (const TA*)gate, sg, gate_bias, ids, (const TA*)table,     \
      vocab, fresh, w, eps, (TO*)out, W)))
    if (cols <= ntv) RESIDUAL_VEC(1);
    else if (cols <= 2 * ntv) RESIDUAL_VEC(2);
    else RESIDUAL_VEC(4);
#undef RESIDUAL_VEC
    MX_RETURN_LAUNCH();
  }
  const int nt = W >= 1024 ? 512 : 256;
  MX_DISPATCH(dt_ab, TA, MX_DISPATCH(dt_out, TO, residual_norm_kernel<TA, TO><<<T, nt, 0, st>>>(
      x, (const TA*)a, sa, (const TA*)b, sb, mult, mult_b, (const TA*)gate, sg, gate_bias, ids,
      (const TA*)table, vocab, fresh, w, eps, (TO*)out, W)));
  MX_RETURN_LAUNCH();
}

// x f32 [T, W].  a given ([T, >= W] slice, row stride sa, type dt_a): x <- x + D1(a); else table given ([vocab, W] of
// type dt_a, ids [T]): x <- D1(scale * table[id]).  Then, with out ([T, W] of type dt_out): out = D2(x).
// D(v) = tanh(alpha v) * w + b elementwise, w and b f32 [W].
MX_API int mx_dyn_tanh(float* x, const void* a, long sa, const int* ids, const void* table, int vocab, float scale,
                       int dt_a, float alpha1, const float* w1, const float* b1, float alpha2, const float* w2,
                       const float* b2, void* out, int dt_out, int T, int W, hipStream_t st) {
  if (T <= 0) return 0;
  if ((a != nullptr || table != nullptr) && (w1 == nullptr || b1 == nullptr)) return (int)hipErrorInvalidValue;
  if (out != nullptr && (w2 == nullptr || b2 == nullptr)) return (int)hipErrorInvalidValue;
  if (table != nullptr && ids == nullptr) return (int)hipErrorInvalidValue;
  const bool vec = W % 4 == 0 && sa % 4 == 0 && ((size_t)a | (size_t)table) % (dt_a == 1 ? 16 : 8) == 0 &&
                   ((size_t)x | (size_t)w1 | (size_t)b1 | (size_t)w2 | (size_t)b2) % 16 == 0 &&
                   (size_t)out % (dt_out == 1 ? 16 : 8) == 0;
  const int cols = vec ? W / 4 : W;
  const int nt = cols >= 256 ? 256 : (cols + 63) / 64 * 64;
  const int rows = T >= 2048 ? 4 : (T >= 1024 ? 2 : 1);
  dim3 grid((T + rows - 1) / rows, (cols + nt - 1) / nt);
  if (vec)
    MX_DISPATCH(dt_a, TA, MX_DISPATCH(dt_out, TO, dyn_tanh_kernel<TA, TO, 4><<<grid, nt, 0, st>>>(
        x, (const TA*)a, sa, ids, (const TA*)table, vocab, scale, alpha1, w1, b1, alpha2, w2, b2, (TO*)out, W, rows, T)));
  else
    MX_DISPATCH(dt_a, TA, MX_DISPATCH(dt_out, TO, dyn_tanh_kernel<TA, TO, 1><<<grid, nt, 0, st>>>(
        x, (const TA*)a, sa, ids, (const TA*)table, vocab, scale, alpha1, w1, b1, alpha2, w2, b2, (TO*)out, W, rows, T)));
  MX_RETURN_LAUNCH();
}

// in [T, groups * n] (row stride si, type dt_in; f32 when dt_in == 1), optional gate of type dt_gate
MX_API int mx_group_norm(const void* in, long si, int dt_in, const void* gate, long sg, int dt_gate, const float* w,
                         float eps, void* out, long so, int dt_out, int T, int groups, int n, hipStream_t st) {
  if (T <= 0) return 0;
  const int nt = n >= 1024 ? 512 : (n >= 256 ? 256 : 64);
  dim3 grid(T, groups);
  MX_DISPATCH(dt_in, TI, MX_DISPATCH(dt_gate, TG, MX_DISPATCH(dt_out, TO, group_norm_kernel<TI, TG, TO>
      <<<grid, nt, 0, st>>>((const TI*)in, si, (const TG*)gate, sg, w, eps, (TO*)out, so, n))));
  MX_RETURN_LAUNCH();
}

MX_API int mx_relu2(const void* in, long si, void* out, long so, int dt, int T, int n, hipStream_t st) {
  const long total = (long)T * n;
  if (total <= 0) return 0;
  const int blocks = (int)((total + 255) / 256 < 16384 ? (total + 255) / 256 : 16384);
  MX_DISPATCH(dt, TT, relu2_kernel<TT><<<blocks, 256, 0, st>>>((const TT*)in, si, (TT*)out, so, n, total));
  MX_RETURN_LAUNCH();
}

MX_API int mx_glu_clamp(const void* gate, long sg, const void* up, long su, float limit, float alpha, void* out,
                        long so, int dt, int T, int n, hipStream_t st) {
  const long total = (long)T * n;
  if (total <= 0) return 0;
  const int V = dt == 1 ? 4 : 8;                       // elements per 16 bytes
  if (n % V == 0 && sg % V == 0 && su % V == 0 && so % V == 0 && ((size_t)gate | (size_t)up | (size_t)out) % 16 == 0 &&
      (size_t)n / V <= 65535u * 256u) {
    const int nv = n / V;
    const int nt = nv >= 256 ? 256 : (nv + 63) / 64 * 64;
    dim3 grid(T, (nv + nt - 1) / nt);
    if (dt == 1)
      glu_clamp_vec_kernel<float, 4><<<grid, nt, 0, st>>>((const float*)gate, sg, (const float*)up, su, limit, alpha,
                                                          (float*)out, so, nv);
    else
      glu_clamp_vec_kernel<bf16, 8><<<grid, nt, 0, st>>>((const bf16*)gate, sg, (const bf16*)up, su, limit, alpha,
                                                         (bf16*)out, so, nv);
    MX_RETURN_LAUNCH();
  }
  const int blocks = (int)((total + 255) / 256 < 16384 ? (total + 255) / 256 : 16384);
  MX_DISPATCH(dt, TT, glu_clamp_kernel<TT><<<blocks, 256, 0, st>>>((const TT*)gate, sg, (const TT*)up, su, limit,
                                                                    alpha, (TT*)out, so, n, total));
  MX_RETURN_LAUNCH();
}

// sigm != 0: sigmoid scores instead of a softmax over the entries; renorm != 0: weights divided by the sum of the
// chosen scores (+ 1e-20); wscale: constant on the weights
MX_API int mx_route_biased(const float* z, const float* bias, int E, int top, int sigm, int renorm, float wscale,
                           float* outw, int* outi, int T, hipStream_t st) {
  if (T <= 0) return 0;
  if (E > 64 * 128 || top > E) return (int)hipErrorInvalidValue;
  route_biased_kernel<<<(T + 3) / 4, 256, 0, st>>>(z, bias, E, top, sigm, renorm, wscale, outw, outi, T);
  MX_RETURN_LAUNCH();
}

MX_API int mx_moe_combine(const void* ys, const int* pos, const int* idx, const float* wts, const void* h, long sh,
                          const void* shared, long ssh, int E, int top, int W, void* out, int dt, int T,
                          hipStream_t st) {
  if (T <= 0) return 0;
  MX_DISPATCH(dt, TT, moe_combine_kernel<TT><<<T, 256, 0, st>>>((const TT*)ys, pos, idx, wts, (const TT*)h, sh,
                                                                (const TT*)shared, ssh, E, top, W, (TT*)out));
  MX_RETURN_LAUNCH();
}
