// tl_norm.hip — the row-wise FP32 steps between the matrix products of a layer-list model. An RMS norm here is
// y = x / sqrt(mean(x^2) + eps) * weight, eps inside the root; "one-plus" weights are stored around zero and applied as
// (1 + w). Norm-first blocks with the Dynamic Tanh norm (tanh(alpha x) * w + b: elementwise, no statistics) need no staged
// row: embedding gather, residual sum and row gather carry the norm of the block that follows in the same pass. One workgroup per token row (256 threads for the rows of a prompt chunk, 1024 for the few rows of a decode step,
// whose launches are nothing but a chain of memory round trips); a row is staged in LDS, so that it is read from memory once.
#include <math.h>

#include "tl_bf16.h"
#include "tl_route.h"
#include "tl_stack.h"

namespace {

constexpr int kMaxWaves = 16;

__device__ __forceinline__ float block_sum(float v, float* red) {  // red: kMaxWaves floats of LDS; result in every thread
#pragma unroll
  for (int o = 32; o >= 1; o >>= 1) v += __shfl_xor(v, o);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.0f;
  for (int w = 0; w < (int)(blockDim.x >> 6); ++w) s += red[w];  // in wave order: the same sum in every thread
  return s;
}

inline int row_threads(int rows) { return rows <= 8 ? 1024 : 256; }

__global__ __launch_bounds__(1024) void embed_norm_kernel(const unsigned short* __restrict__ table, int vocab, int width,
                                                         const int* __restrict__ tokens, const float* __restrict__ w,
                                                         float eps, float* __restrict__ x) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[kMaxWaves];
  const int t = blockIdx.x, tok = tokens[t];
  const bool in = tok >= 0 && tok < vocab;
  const unsigned short* e = table + (size_t)(in ? tok : 0) * width;
  float ss = 0.0f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = in ? __uint_as_float((unsigned)e[c] << 16) : 0.0f;
    row[c] = v;
    ss += v * v;
  }
  ss = block_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)width + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x) x[(size_t)t * width + c] = row[c] * inv * (1.0f + w[c]);
}

__global__ __launch_bounds__(1024) void qkv_post_kernel(const QkvPostArgs a) {
  __shared__ float red[kMaxWaves];
  const int t = blockIdx.x;
  const int pos = (a.pos_dev ? *a.pos_dev : a.start_pos) + t;
  float* q = a.qkv + (size_t)t * a.ld;
  const float* k = q + a.qd;
  const float* v = k + a.kd;
  if (a.head_dim > 0) {  // every block of head_dim of q and of k on its own, one weight vector each: a wave per block in turn
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nw = blockDim.x >> 6, hd = a.head_dim;
    const int nq = a.qd / hd, nk = a.kd / hd;
    float* kr = a.kc + (size_t)pos * a.kd;
    for (int g = wave; g < nq + nk; g += nw) {
      const bool isq = g < nq;
      const float* src = isq ? q + (size_t)g * hd : k + (size_t)(g - nq) * hd;
      float* dst = isq ? q + (size_t)g * hd : kr + (size_t)(g - nq) * hd;
      const float* w = isq ? a.q_norm : a.k_norm;
      float ss = 0.0f;
      for (int d = lane; d < hd; d += 64) ss += src[d] * src[d];
      ss = tl_wave_sum(ss);
      const float inv = 1.0f / sqrtf(ss / (float)hd + a.eps);
      for (int d = lane; d < hd; d += 64) dst[d] = src[d] * inv * w[d];
    }
    float* vr = a.vc + (size_t)pos * a.vd;
    for (int c = threadIdx.x; c < a.vd; c += blockDim.x) vr[c] = v[c];
    return;
  }
  float sq = 0.0f, sk = 0.0f;
  if (a.q_norm)
    for (int c = threadIdx.x; c < a.qd; c += blockDim.x) sq += q[c] * q[c];
  if (a.k_norm)
    for (int c = threadIdx.x; c < a.kd; c += blockDim.x) sk += k[c] * k[c];
  sq = block_sum(sq, red);
  sk = block_sum(sk, red);
  if (a.q_norm) {
    const float inv = 1.0f / sqrtf(sq / (float)a.qd + a.eps);
    for (int c = threadIdx.x; c < a.qd; c += blockDim.x) q[c] = q[c] * inv * a.q_norm[c];
  }
  if (a.q_temp_every > 0) {  // query temperature: grows by the logarithm of the position, in steps of q_temp_every positions
    const float f = 1.0f + a.q_temp_coef * logf((float)((pos + 1) / a.q_temp_every) + 1.0f);
    for (int c = threadIdx.x; c < a.qd; c += blockDim.x) q[c] *= f;
  }
  {
    const float inv = a.k_norm ? 1.0f / sqrtf(sk / (float)a.kd + a.eps) : 1.0f;
    float* kr = a.kc + (size_t)pos * a.kd;
    for (int c = threadIdx.x; c < a.kd; c += blockDim.x) kr[c] = a.k_norm ? k[c] * inv * a.k_norm[c] : k[c];
  }
  float* vr = a.vc + (size_t)pos * a.vd;
  if (a.vmix == 2) {
    const float lam = *a.lambda;
    const float* vf = a.v_first + (size_t)t * a.vd;
    for (int c = threadIdx.x; c < a.vd; c += blockDim.x) vr[c] = (1.0f - lam) * v[c] + lam * vf[c];
  } else {
    float* vf = a.vmix == 1 ? a.v_first + (size_t)t * a.vd : nullptr;
    for (int c = threadIdx.x; c < a.vd; c += blockDim.x) {
      vr[c] = v[c];
      if (vf) vf[c] = v[c];
    }
  }
}

__global__ __launch_bounds__(1024) void resid_norm_kernel(const ResidNormArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[kMaxWaves];
  const int t = blockIdx.x;
  float ss = 0.0f;
  for (int c = threadIdx.x; c < a.width; c += blockDim.x) {
    float y = a.a ? a.a[(size_t)t * a.width + c] : 0.0f;
    if (a.slots) {
      float e = 0.0f;
      for (int j = 0; j < a.top; ++j) e += a.slot_w[t * a.top + j] * a.slots[((size_t)t * a.top + j) * a.width + c];
      y += e;
    }
    row[c] = y;
    ss += y * y;
  }
  ss = block_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)a.width + a.eps);
  float* x = a.x + (size_t)t * a.width;
  for (int c = threadIdx.x; c < a.width; c += blockDim.x) {
    const float xn = x[c] + row[c] * inv * (1.0f + a.w[c]);
    x[c] = xn;
    row[c] = xn;  // the updated row stays in LDS for the router below
  }
  if (!a.route.w) return;
  // ---- the router of the feed-forward that follows: logits = W_r x + b over the row in LDS, a wave per expert in turn ----
  __syncthreads();
  float* z = row + ((a.width + 3) & ~3);  // [experts]
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nwaves = blockDim.x >> 6;
  const bool vec = (a.width & 7) == 0 && ((size_t)a.route.w & 15) == 0;
  for (int e = wave; e < a.route.experts; e += nwaves) {
    float sdot;
    tl_wave_dot_rows<1>(a.route.w + (size_t)e * a.width, 0, 1, row, a.width, vec, lane, &sdot);
    if (lane == 0) z[e] = sdot + (a.route.b ? a.route.b[e] : 0.0f);
  }
  __syncthreads();
  if (wave == 0)
    tl_route_select(z, a.route.experts, a.route.top, a.route.ids + (size_t)t * a.route.top, a.route.wts + (size_t)t * a.route.top, lane);
}

__global__ __launch_bounds__(1024) void norm_rows_kernel(const float* __restrict__ x, int width, const int* __restrict__ rows,
                                                        const float* __restrict__ w, float eps, float* __restrict__ out,
                                                        float w_add) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[kMaxWaves];
  const int i = blockIdx.x;
  const float* xr = x + (size_t)(rows ? rows[i] : i) * width;
  float ss = 0.0f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = xr[c];
    row[c] = v;
    ss += v * v;
  }
  ss = block_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)width + eps);
  for (int c = threadIdx.x; c < width; c += blockDim.x) out[(size_t)i * width + c] = row[c] * inv * (w_add + w[c]);
}

// the router of the feed-forward that reads the finished row in LDS: logits, a wave per expert in turn, then the selection
__device__ __forceinline__ void route_row(const RouterArgs& r, float* row, int width, int t) {
  __syncthreads();
  float* z = row + ((width + 3) & ~3);  // [experts] (+ [experts] keys + [groups] for the group-ranked kinds)
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nwaves = blockDim.x >> 6;
  const bool vec = (width & 7) == 0 && ((size_t)r.w & 15) == 0;
  for (int e = wave; e < r.experts; e += nwaves) {
    float sdot;
    tl_wave_dot_rows<1>(r.w + (size_t)e * width, 0, 1, row, width, vec, lane, &sdot);
    if (lane == 0) z[e] = sdot + (r.b ? r.b[e] : 0.0f);
  }
  __syncthreads();
  if (wave == 0) tl_route_token(r, z, t, lane);
}

// pre-norm blocks with an RMS norm: the residual sum and the norm of what reads x next
__global__ __launch_bounds__(1024) void resid_rms_kernel(const ResidRmsArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[kMaxWaves];
  const int t = blockIdx.x;
  float* xr = a.x + (size_t)t * a.width;
  const bool add = a.a || a.b || a.slots;
  float ss = 0.0f;
  for (int c = threadIdx.x; c < a.width; c += blockDim.x) {
    float v = xr[c];
    if (add) {
      float y = a.a ? a.a_scale * a.a[(size_t)t * a.width + c] : 0.0f;
      if (a.b) y += a.b_scale * a.b[(size_t)t * a.width + c];
      if (a.slots) {
        float e = 0.0f;
        for (int j = 0; j < a.top; ++j) e += a.slot_w[t * a.top + j] * a.slots[((size_t)t * a.top + j) * a.width + c];
        y += e;
      }
      v += y;
      xr[c] = v;
    }
    row[c] = v;
    ss += v * v;
  }
  if (!a.w) return;
  ss = block_sum(ss, red);
  const float inv = 1.0f / sqrtf(ss / (float)a.width + a.eps), w_add = a.one_plus ? 1.0f : 0.0f;
  if (!a.canon_w) {
    for (int c = threadIdx.x; c < a.width; c += blockDim.x) {
      const float hv = row[c] * inv * (w_add + a.w[c]);
      a.h[(size_t)t * a.width + c] = hv;
      row[c] = hv;  // (own columns only) what the sublayer reads stays in LDS for the router below
    }
  } else {
    const int H = a.canon_taps - 1;  // (one token: the launcher checks)
    for (int c = threadIdx.x; c < a.width; c += blockDim.x) {
      const float cur = row[c] * inv * (w_add + a.w[c]);
      const unsigned short* w = a.canon_w + (size_t)c * a.canon_taps;
      float acc = tl_bf2f(w[H]) * cur;
      for (int j = 0; j < H; ++j) {
        const float u = a.canon_hist[(size_t)j * a.width + c];
        acc += tl_bf2f(w[j]) * u;
        if (j > 0) a.canon_hist[(size_t)(j - 1) * a.width + c] = u;
      }
      if (H > 0) a.canon_hist[(size_t)(H - 1) * a.width + c] = cur;
      a.h[c] = cur + acc;
      row[c] = cur + acc;
    }
  }
  if (!a.route.w) return;
  route_row(a.route, row, a.width, t);
}

constexpr int kMaxRowFloats = 16 * 1024;  // 64 KB of LDS for the staged row

// ---- layer norm: mean, then the mean of the squared deviations, both over the row staged in LDS (two passes, FP32) ----------
// row[] holds the input; every thread returns with (mean, 1 / sqrt(var + eps))
__device__ __forceinline__ void ln_stats(const float* row, int width, float eps, float* red, float* mean, float* inv) {
  float sm = 0.0f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) sm += row[c];
  const float mu = block_sum(sm, red) / (float)width;
  float sv = 0.0f;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float d = row[c] - mu;
    sv += d * d;
  }
  const float var = block_sum(sv, red) / (float)width;
  *mean = mu;
  *inv = 1.0f / sqrtf(var + eps);
}

__global__ __launch_bounds__(1024) void embed_ln_kernel(const unsigned short* __restrict__ table, int vocab, int width,
                                                       const int* __restrict__ tokens, const LnParams emb, const LnParams next,
                                                       float eps, float* __restrict__ x, float* __restrict__ h) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[kMaxWaves];
  const int t = blockIdx.x, tok = tokens[t];
  const bool in = tok >= 0 && tok < vocab;
  const unsigned short* e = table + (size_t)(in ? tok : 0) * width;
  for (int c = threadIdx.x; c < width; c += blockDim.x) row[c] = in ? __uint_as_float((unsigned)e[c] << 16) : 0.0f;
  __syncthreads();
  float mu, inv;
  if (emb.w) {
    ln_stats(row, width, eps, red, &mu, &inv);
    for (int c = threadIdx.x; c < width; c += blockDim.x) row[c] = (row[c] - mu) * inv * emb.w[c] + (emb.b ? emb.b[c] : 0.0f);  // own columns only
    __syncthreads();
  }
  for (int c = threadIdx.x; c < width; c += blockDim.x) x[(size_t)t * width + c] = row[c];
  if (!next.w) return;
  ln_stats(row, width, eps, red, &mu, &inv);
  for (int c = threadIdx.x; c < width; c += blockDim.x) h[(size_t)t * width + c] = (row[c] - mu) * inv * next.w[c] + (next.b ? next.b[c] : 0.0f);
}

__global__ __launch_bounds__(1024) void resid_ln_kernel(float* __restrict__ x, const float* __restrict__ a, int width,
                                                       const LnParams next, float eps, float* __restrict__ h) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[kMaxWaves];
  const int t = blockIdx.x;
  float* xr = x + (size_t)t * width;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    const float v = xr[c] + a[(size_t)t * width + c];
    xr[c] = v;
    row[c] = v;
  }
  if (!next.w) return;
  __syncthreads();
  float mu, inv;
  ln_stats(row, width, eps, red, &mu, &inv);
  for (int c = threadIdx.x; c < width; c += blockDim.x) h[(size_t)t * width + c] = (row[c] - mu) * inv * next.w[c] + (next.b ? next.b[c] : 0.0f);
}

__global__ __launch_bounds__(1024) void ln_rows_kernel(const float* __restrict__ x, int width, const int* __restrict__ rows,
                                                      const LnParams p, float eps, float* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[kMaxWaves];
  const int i = blockIdx.x;
  const float* xr = x + (size_t)(rows ? rows[i] : i) * width;
  for (int c = threadIdx.x; c < width; c += blockDim.x) row[c] = xr[c];
  __syncthreads();
  float mu, inv;
  ln_stats(row, width, eps, red, &mu, &inv);
  for (int c = threadIdx.x; c < width; c += blockDim.x) out[(size_t)i * width + c] = (row[c] - mu) * inv * p.w[c] + (p.b ? p.b[c] : 0.0f);
}

// ---- residual streams: write-back of a sublayer into every stream, the next sublayer's input and its layer norm, one workgroup
// per token. V columns at a time per thread (16-byte accesses); S streams (0: a.streams of them, at most kMaxStreams) -----------
constexpr int kMaxStreams = 16;

template <int V>
struct HyperVec {
  float v[V];
  __device__ __forceinline__ void load(const float* p) {
    if constexpr (V == 4) {
      const float4 f = *reinterpret_cast<const float4*>(p);
      v[0] = f.x, v[1] = f.y, v[2] = f.z, v[3] = f.w;
    } else {
      v[0] = p[0];
    }
  }
  __device__ __forceinline__ void store(float* p) const {
    if constexpr (V == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    else p[0] = v[0];
  }
};

template <int S, int V>
__global__ __launch_bounds__(1024) void hyper_kernel(const HyperArgs a) {
  extern __shared__ __attribute__((aligned(16))) float row[];
  __shared__ float red[kMaxWaves], cf[kMaxStreams * (kMaxStreams + 2)];
  constexpr int SM = S > 0 ? S : kMaxStreams;
  const int ns = S > 0 ? S : a.streams, t = blockIdx.x;
  float* xr = a.x + (size_t)t * ns * a.width;
  const bool add = a.a || a.slots;
  // coefficients: mix [from][to] | mult * out [to] | in [from]
  for (int i = threadIdx.x; i < ns * ns; i += blockDim.x) cf[i] = a.mix ? a.mix[i] : (i / ns == i % ns ? 1.0f : 0.0f);
  for (int i = threadIdx.x; i < ns; i += blockDim.x) {
    cf[ns * ns + i] = a.mult * (a.out ? a.out[i] : 1.0f);
    cf[ns * ns + ns + i] = a.in ? a.in[i] : 1.0f;
  }
  __syncthreads();
  int tok = 0;
  bool known = true;
  if (a.table) {
    tok = a.tokens[t];
    known = tok >= 0 && tok < a.vocab;
  }
  const unsigned short* er = a.table ? a.table + (size_t)(known ? tok : 0) * a.width : nullptr;
  for (int c = threadIdx.x * V; c < a.width; c += blockDim.x * V) {
    HyperVec<V> x[SM];
    if (a.table) {
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float v = known ? tl_bf2f(er[c + e]) * a.embed_scale : 0.0f;  // (an id outside the table embeds as zeros)
#pragma unroll
        for (int s = 0; s < SM; ++s) x[s].v[e] = v;
      }
    } else {
#pragma unroll
      for (int s = 0; s < SM; ++s)
        if (s < ns) x[s].load(xr + (size_t)s * a.width + c);
    }
    if (add) {
      HyperVec<V> y;
#pragma unroll
      for (int e = 0; e < V; ++e) y.v[e] = 0.0f;
      if (a.a) y.load(a.a + (size_t)t * a.width + c);
      if (a.slots) {
        HyperVec<V> es;
#pragma unroll
        for (int e = 0; e < V; ++e) es.v[e] = 0.0f;
        for (int j = 0; j < a.top; ++j) {
          HyperVec<V> o;
          o.load(a.slots + ((size_t)t * a.top + j) * a.width + c);
          const float w = a.slot_w[t * a.top + j];
#pragma unroll
          for (int e = 0; e < V; ++e) es.v[e] += w * o.v[e];
        }
#pragma unroll
        for (int e = 0; e < V; ++e) y.v[e] += es.v[e];
      }
      HyperVec<V> n[SM];
#pragma unroll
      for (int o = 0; o < SM; ++o) {
        if (o >= ns) continue;
#pragma unroll
        for (int e = 0; e < V; ++e) n[o].v[e] = cf[ns * ns + o] * y.v[e];
#pragma unroll
        for (int s = 0; s < SM; ++s) {
          if (s >= ns) continue;
          const float m = cf[s * ns + o];
#pragma unroll
          for (int e = 0; e < V; ++e) n[o].v[e] += m * x[s].v[e];
        }
      }
#pragma unroll
      for (int s = 0; s < SM; ++s)
        if (s < ns) x[s] = n[s];
    }
    HyperVec<V> u, sm;
#pragma unroll
    for (int e = 0; e < V; ++e) u.v[e] = sm.v[e] = 0.0f;
#pragma unroll
    for (int s = 0; s < SM; ++s) {
      if (s >= ns) continue;
      if (add || a.table) x[s].store(xr + (size_t)s * a.width + c);
      const float w = cf[ns * ns + ns + s];
#pragma unroll
      for (int e = 0; e < V; ++e) {
        u.v[e] += w * x[s].v[e];
        sm.v[e] += x[s].v[e];
      }
    }
    if (a.sum) sm.store(a.sum + (size_t)t * a.width + c);
    u.store(row + c);
  }
  if (!a.next.w) return;
  __syncthreads();
  float mu, inv;
  ln_stats(row, a.width, a.eps, red, &mu, &inv);
  for (int c = threadIdx.x; c < a.width; c += blockDim.x) {
    const float v = (row[c] - mu) * inv * a.next.w[c] + (a.next.b ? a.next.b[c] : 0.0f);
    a.h[(size_t)t * a.width + c] = v;
    row[c] = v;  // (own columns only) stays for the router below
  }
  if (!a.route.w) return;
  route_row(a.route, row, a.width, t);
}

template <int V>
void launch_hyper(const HyperArgs& a, size_t lds, hipStream_t s) {
  const int th = row_threads(a.T);
  switch (a.streams) {
    case 1: hyper_kernel<1, V><<<a.T, th, lds, s>>>(a); break;
    case 2: hyper_kernel<2, V><<<a.T, th, lds, s>>>(a); break;
    case 3: hyper_kernel<3, V><<<a.T, th, lds, s>>>(a); break;
    case 4: hyper_kernel<4, V><<<a.T, th, lds, s>>>(a); break;
    default: hyper_kernel<0, 1><<<a.T, th, lds, s>>>(a); break;
  }
}

// ---- two sublayers that read the same x: both outputs (normed on the way in, if asked for) join the residual, and the norms of the
// two sublayers that read x next share one set of statistics. A thread holds its columns (PER pieces of V) in registers ----------
__device__ __forceinline__ void block_sum2(float& p, float& q, float* red) {  // red: 2 kMaxWaves floats
#pragma unroll
  for (int o = 32; o >= 1; o >>= 1) {
    p += __shfl_xor(p, o);
    q += __shfl_xor(q, o);
  }
  if ((threadIdx.x & 63) == 0) {
    red[threadIdx.x >> 6] = p;
    red[kMaxWaves + (threadIdx.x >> 6)] = q;
  }
  __syncthreads();
  p = q = 0.0f;
  for (int w = 0; w < (int)(blockDim.x >> 6); ++w) {
    p += red[w];
    q += red[kMaxWaves + w];
  }
}

template <int V, int PER>
__global__ __launch_bounds__(1024) void resid_norms_kernel(const ResidNormsArgs a) {
  __shared__ float red[2 * kMaxWaves], red2[kMaxWaves];
  const size_t r0 = (size_t)blockIdx.x * a.width;
  const int step = blockDim.x * V, c0 = threadIdx.x * V;
  HyperVec<V> x[PER], ya[PER], yb[PER];
  float sa = 0.0f, sb = 0.0f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = c0 + i * step;
#pragma unroll
    for (int e = 0; e < V; ++e) x[i].v[e] = ya[i].v[e] = yb[i].v[e] = 0.0f;
    if (c >= a.width) continue;
    x[i].load(a.x + r0 + c);
    if (a.a) ya[i].load(a.a + r0 + c);
    if (a.b) yb[i].load(a.b + r0 + c);
    if (a.c) {
      HyperVec<V> yc;
      yc.load(a.c + r0 + c);
#pragma unroll
      for (int e = 0; e < V; ++e) x[i].v[e] += yc.v[e];
    }
#pragma unroll
    for (int e = 0; e < V; ++e) {
      sa += ya[i].v[e] * ya[i].v[e];
      sb += yb[i].v[e] * yb[i].v[e];
    }
  }
  float fa = a.a_scale, fb = a.b_scale;
  if (a.a_w || a.b_w) {
    block_sum2(sa, sb, red);
    if (a.a_w) fa *= 1.0f / sqrtf(sa / (float)a.width + a.eps);
    if (a.b_w) fb *= 1.0f / sqrtf(sb / (float)a.width + a.eps);
  }
  float ss = 0.0f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = c0 + i * step;
    if (c >= a.width) continue;
    if (a.a) {
      HyperVec<V> w;
#pragma unroll
      for (int e = 0; e < V; ++e) w.v[e] = 1.0f;
      if (a.a_w) w.load(a.a_w + c);
#pragma unroll
      for (int e = 0; e < V; ++e) x[i].v[e] += ya[i].v[e] * fa * w.v[e];
    }
    if (a.b) {
      HyperVec<V> w;
#pragma unroll
      for (int e = 0; e < V; ++e) w.v[e] = 1.0f;
      if (a.b_w) w.load(a.b_w + c);
#pragma unroll
      for (int e = 0; e < V; ++e) x[i].v[e] += yb[i].v[e] * fb * w.v[e];
    }
    if (a.a || a.b || a.c) x[i].store(a.x + r0 + c);
#pragma unroll
    for (int e = 0; e < V; ++e) ss += x[i].v[e] * x[i].v[e];
  }
  if (!a.w1 && !a.w2) return;
  const float inv = 1.0f / sqrtf(block_sum(ss, red2) / (float)a.width + a.eps);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = c0 + i * step;
    if (c >= a.width) continue;
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const float* wp = k == 0 ? a.w1 : a.w2;
      if (!wp) continue;
      HyperVec<V> w;
      w.load(wp + c);
#pragma unroll
      for (int e = 0; e < V; ++e) w.v[e] *= x[i].v[e] * inv;
      w.store((k == 0 ? a.h1 : a.h2) + r0 + c);
    }
  }
}

__device__ __forceinline__ float dyt_of(float x, float alpha, float w, float b) { return tanhf(alpha * x) * w + b; }

// grid (column blocks of 256, T)
__global__ __launch_bounds__(256) void embed_rows_kernel(const unsigned short* __restrict__ table, int vocab, int width,
                                                        const int* __restrict__ tokens, float* __restrict__ x,
                                                        const DytParams next, float* __restrict__ h, float scale) {
  const int t = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= width) return;
  const int tok = tokens[t];
  const float v = (tok >= 0 && tok < vocab) ? __uint_as_float((unsigned)table[(size_t)tok * width + c] << 16) * scale : 0.0f;
  x[(size_t)t * width + c] = v;
  if (next.alpha) h[(size_t)t * width + c] = dyt_of(v, *next.alpha, next.w[c], next.b[c]);
}

__global__ __launch_bounds__(256) void resid_sum_kernel(const ResidSumArgs a) {
  const int t = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= a.width) return;
  const size_t i = (size_t)t * a.width + c;
  float y = a.a ? a.a[i] : 0.0f;
  if (a.slots) {
    float e = 0.0f;
    for (int j = 0; j < a.top; ++j) e += a.slot_w[t * a.top + j] * a.slots[((size_t)t * a.top + j) * a.width + c];
    y += e;
  }
  if (a.b) y += a.b_gate ? a.b_gate[t] * a.b[i] : a.b[i];
  const float xn = a.x[i] + y;
  a.x[i] = xn;
  if (a.next.alpha) a.h[i] = dyt_of(xn, *a.next.alpha, a.next.w[c], a.next.b[c]);
}

__global__ __launch_bounds__(256) void dyt_rows_kernel(const float* __restrict__ x, int width, const int* __restrict__ rows,
                                                      const DytParams p, float* __restrict__ out) {
  const int i = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  if (c >= width) return;
  out[(size_t)i * width + c] = dyt_of(x[(size_t)(rows ? rows[i] : i) * width + c], *p.alpha, p.w[c], p.b[c]);
}

}  // namespace

int tl_launch_embed_rows(const uint16_t* table, int vocab, int width, const int* tokens_dev, int T, float* x, const DytParams& next,
                         float* h, hipStream_t s, float scale) {
  TL_REQUIRE(table && tokens_dev && x && T > 0 && T <= 65535 && vocab > 0 && width > 0, "embed_rows: bad arguments");
  TL_REQUIRE(!next.alpha || (next.w && next.b && h), "embed_rows: a norm without its weights or output");
  embed_rows_kernel<<<dim3((width + 255) / 256, T), 256, 0, s>>>(table, vocab, width, tokens_dev, x, next, h, scale);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_resid_sum(const ResidSumArgs& a, hipStream_t s) {
  TL_REQUIRE(a.x && a.T > 0 && a.T <= 65535 && a.width > 0 && (a.a || a.b || a.slots), "resid_sum: bad arguments");
  TL_REQUIRE(!a.slots || (a.slot_w && a.top > 0), "resid_sum: expert slots without weights");
  TL_REQUIRE(!a.next.alpha || (a.next.w && a.next.b && a.h), "resid_sum: a norm without its weights or output");
  resid_sum_kernel<<<dim3((a.width + 255) / 256, a.T), 256, 0, s>>>(a);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_dyt_rows(const float* x, int width, const int* rows_dev, int n, const DytParams& p, float* out, hipStream_t s) {
  TL_REQUIRE(x && out && p.alpha && p.w && p.b && n > 0 && n <= 65535 && width > 0, "dyt_rows: bad arguments");
  dyt_rows_kernel<<<dim3((width + 255) / 256, n), 256, 0, s>>>(x, width, rows_dev, p, out);
  TL_HIP(hipGetLastError());
  return 0;
}

extern "C" int tl_dyt_norm(const float* x_dev, const float* alpha_dev, const float* weight_dev, const float* bias_dev,
                           float* out_dev, int num_tokens, int width, void* stream) {
  DytParams p = {alpha_dev, weight_dev, bias_dev};
  return tl_launch_dyt_rows(x_dev, width, nullptr, num_tokens, p, out_dev, static_cast<hipStream_t>(stream));
}

int tl_launch_embed_ln(const uint16_t* table, int vocab, int width, const int* tokens_dev, int T, const LnParams& emb,
                       const LnParams& next, float eps, float* x, float* h, hipStream_t s) {
  TL_REQUIRE(table && tokens_dev && x && T > 0 && vocab > 0, "embed_ln: bad arguments");
  TL_REQUIRE(width > 0 && width <= kMaxRowFloats, "embed_ln: width %d outside (0, %d]", width, kMaxRowFloats);
  TL_REQUIRE(!next.w || h, "embed_ln: a norm without its output");
  embed_ln_kernel<<<T, row_threads(T), sizeof(float) * width, s>>>(table, vocab, width, tokens_dev, emb, next, eps, x, h);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_resid_ln(float* x, const float* a, int T, int width, const LnParams& next, float eps, float* h, hipStream_t s) {
  TL_REQUIRE(x && a && T > 0, "resid_ln: bad arguments");
  TL_REQUIRE(width > 0 && width <= kMaxRowFloats, "resid_ln: width %d outside (0, %d]", width, kMaxRowFloats);
  TL_REQUIRE(!next.w || h, "resid_ln: a norm without its output");
  resid_ln_kernel<<<T, row_threads(T), sizeof(float) * width, s>>>(x, a, width, next, eps, h);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_ln_rows(const float* x, int width, const int* rows_dev, int n, const LnParams& p, float eps, float* out,
                      hipStream_t s) {
  TL_REQUIRE(x && out && p.w && n > 0, "ln_rows: bad arguments");
  TL_REQUIRE(width > 0 && width <= kMaxRowFloats, "ln_rows: width %d outside (0, %d]", width, kMaxRowFloats);
  ln_rows_kernel<<<n, row_threads(n), sizeof(float) * width, s>>>(x, width, rows_dev, p, eps, out);
  TL_HIP(hipGetLastError());
  return 0;
}

extern "C" int tl_layer_norm(const float* x_dev, const float* weight_dev, const float* bias_dev, float* out_dev, int num_tokens,
                             int width, float eps, void* stream) {
  return tl_launch_ln_rows(x_dev, width, nullptr, num_tokens, LnParams{weight_dev, bias_dev}, eps, out_dev,
                           static_cast<hipStream_t>(stream));
}

int tl_launch_embed_norm(const uint16_t* table, int vocab, int width, const int* tokens_dev, int T, const float* w, float eps,
                         float* x, hipStream_t s) {
  TL_REQUIRE(table && tokens_dev && w && x && T > 0 && vocab > 0, "embed_norm: bad arguments");
  TL_REQUIRE(width > 0 && width <= kMaxRowFloats, "embed_norm: width %d outside (0, %d]", width, kMaxRowFloats);
  embed_norm_kernel<<<T, row_threads(T), sizeof(float) * width, s>>>(table, vocab, width, tokens_dev, w, eps, x);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_qkv_post(const QkvPostArgs& a, hipStream_t s) {
  TL_REQUIRE(a.qkv && a.kc && a.vc && a.T > 0 && a.qd > 0 && a.kd > 0 && a.vd > 0 && a.ld >= a.qd + a.kd + a.vd,
             "qkv_post: bad arguments");
  TL_REQUIRE(a.vmix == 0 || a.v_first, "qkv_post: value mixing without a v_first buffer");
  TL_REQUIRE(a.vmix != 2 || a.lambda, "qkv_post: value mixing without its coefficient");
  TL_REQUIRE(a.head_dim == 0 || (a.head_dim > 0 && a.qd % a.head_dim == 0 && a.kd % a.head_dim == 0 && a.q_norm && a.k_norm &&
                                 a.vmix == 0 && a.q_temp_every == 0),
             "qkv_post: a norm per block of %d over %d / %d", a.head_dim, a.qd, a.kd);
  qkv_post_kernel<<<a.T, row_threads(a.T), 0, s>>>(a);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_resid_norm(const ResidNormArgs& a, hipStream_t s) {
  TL_REQUIRE(a.x && a.w && a.T > 0 && (a.a || a.slots), "resid_norm: bad arguments");
  TL_REQUIRE(a.width > 0 && a.width <= kMaxRowFloats, "resid_norm: width %d outside (0, %d]", a.width, kMaxRowFloats);
  TL_REQUIRE(!a.slots || (a.slot_w && a.top > 0), "resid_norm: expert slots without weights");
  size_t lds = sizeof(float) * a.width;
  if (a.route.w) {
    TL_REQUIRE(a.route.ids && a.route.wts && a.route.experts > 0 && a.route.top > 0 && a.route.top <= a.route.experts,
               "resid_norm: bad router arguments");
    lds = sizeof(float) * (((a.width + 3) & ~3) + a.route.experts);
    TL_REQUIRE(lds <= 64 * 1024, "resid_norm: width %d + %d experts do not fit the staged row", a.width, a.route.experts);
  }
  resid_norm_kernel<<<a.T, row_threads(a.T), lds, s>>>(a);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_resid_rms(const ResidRmsArgs& a, hipStream_t s) {
  TL_REQUIRE(a.x && a.T > 0 && (a.w || a.a || a.b || a.slots), "resid_rms: bad arguments");
  TL_REQUIRE(a.width > 0 && a.width <= kMaxRowFloats, "resid_rms: width %d outside (0, %d]", a.width, kMaxRowFloats);
  TL_REQUIRE(!a.slots || (a.slot_w && a.top > 0), "resid_rms: expert slots without weights");
  TL_REQUIRE(!a.w || a.h, "resid_rms: a norm without its output");
  TL_REQUIRE(!a.canon_w || (a.T == 1 && a.w && a.canon_taps >= 1 && (a.canon_taps == 1 || a.canon_hist)),
             "resid_rms: the convolution rides along for one token behind a norm (%d tokens, %d taps)", a.T, a.canon_taps);
  size_t lds = sizeof(float) * a.width;
  if (a.route.w) {
    const RouterArgs& r = a.route;
    TL_REQUIRE(a.w && r.ids && r.wts && r.experts > 0 && r.top > 0 && r.top <= r.experts && !r.gate_w,
               "resid_rms: bad router arguments");
    TL_REQUIRE(r.kind == TL_ROUTE_TOP_LOGITS || r.kind == TL_ROUTE_SOFTMAX || (r.groups > 0 && r.experts % r.groups == 0 && r.keep > 0 && r.keep <= r.groups &&
                                                  (long long)r.keep * (r.experts / r.groups) >= r.top),
               "resid_rms: %d experts in %d groups, %d kept, top %d", r.experts, r.groups, r.keep, r.top);
    lds = sizeof(float) * (((a.width + 3) & ~3) + 2 * (size_t)r.experts + (r.groups > 0 ? r.groups : 0));
    TL_REQUIRE(lds <= 64 * 1024, "resid_rms: width %d + %d experts do not fit the staged row", a.width, r.experts);
  }
  resid_rms_kernel<<<a.T, row_threads(a.T), lds, s>>>(a);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_resid_norms(const ResidNormsArgs& a, hipStream_t s) {
  TL_REQUIRE(a.x && a.T > 0 && (a.w1 || a.w2 || a.a || a.b || a.c), "resid_norms: bad arguments");
  TL_REQUIRE(a.width > 0 && a.width <= kMaxRowFloats, "resid_norms: width %d outside (0, %d]", a.width, kMaxRowFloats);
  TL_REQUIRE((!a.w1 || a.h1) && (!a.w2 || a.h2), "resid_norms: a norm without its output");
  TL_REQUIRE((!a.a_w || a.a) && (!a.b_w || a.b), "resid_norms: norm weights without a sublayer output");
  bool v4 = (a.width & 3) == 0;
  for (const float* p : {(const float*)a.x, a.a, a.a_w, a.b, a.b_w, a.c, a.w1, a.w2, (const float*)a.h1, (const float*)a.h2})
    v4 = v4 && ((size_t)p & 15) == 0;
  const int pieces = v4 ? a.width / 4 : a.width, most = v4 ? 4 : 16;
  int th = row_threads(a.T);
  while (th < 1024 && (pieces + th - 1) / th > most) th *= 2;
  const int per = (pieces + th - 1) / th;
  if (v4) {
    if (per <= 1) resid_norms_kernel<4, 1><<<a.T, th, 0, s>>>(a);
    else if (per <= 2) resid_norms_kernel<4, 2><<<a.T, th, 0, s>>>(a);
    else resid_norms_kernel<4, 4><<<a.T, th, 0, s>>>(a);
  } else {
    if (per <= 4) resid_norms_kernel<1, 4><<<a.T, th, 0, s>>>(a);
    else resid_norms_kernel<1, 16><<<a.T, th, 0, s>>>(a);
  }
  TL_HIP(hipGetLastError());
  return 0;
}

extern "C" int tl_resid_two_norms(float* x_dev, const float* a_dev, float a_scale, const float* a_weight_dev, const float* b_dev,
                                  float b_scale, const float* b_weight_dev, const float* c_dev, const float* weight1_dev,
                                  float* h1_dev, const float* weight2_dev, float* h2_dev, int num_tokens, int width, float eps,
                                  void* stream) {
  ResidNormsArgs a = {};
  a.x = x_dev;
  a.T = num_tokens;
  a.width = width;
  a.a = a_dev;
  a.a_w = a_weight_dev;
  a.a_scale = a_scale;
  a.b = b_dev;
  a.b_w = b_weight_dev;
  a.b_scale = b_scale;
  a.c = c_dev;
  a.w1 = weight1_dev;
  a.w2 = weight2_dev;
  a.h1 = h1_dev;
  a.h2 = h2_dev;
  a.eps = eps;
  return tl_launch_resid_norms(a, static_cast<hipStream_t>(stream));
}

int tl_launch_norm_rows(const float* x, int width, const int* rows_dev, int n, const float* w, float eps, float* out,
                        hipStream_t s, int one_plus) {
  TL_REQUIRE(x && w && out && n > 0, "norm_rows: bad arguments");
  TL_REQUIRE(width > 0 && width <= kMaxRowFloats, "norm_rows: width %d outside (0, %d]", width, kMaxRowFloats);
  norm_rows_kernel<<<n, row_threads(n), sizeof(float) * width, s>>>(x, width, rows_dev, w, eps, out, one_plus ? 1.0f : 0.0f);
  TL_HIP(hipGetLastError());
  return 0;
}

extern "C" int tl_resid_rmsnorm(float* x_dev, const float* y_dev, const float* weight_dev, int num_tokens, int width, float eps,
                                void* stream) {
  ResidNormArgs a = {};
  a.x = x_dev;
  a.T = num_tokens;
  a.width = width;
  a.a = y_dev;
  a.w = weight_dev;
  a.eps = eps;
  return tl_launch_resid_norm(a, static_cast<hipStream_t>(stream));
}

int tl_launch_hyper(const HyperArgs& a, hipStream_t s) {
  TL_REQUIRE(a.x && a.T > 0 && (a.a || a.slots || a.table || a.sum || a.next.w), "hyper: bad arguments");
  TL_REQUIRE(a.streams >= 1 && a.streams <= kMaxStreams, "hyper: %d streams outside [1, %d]", a.streams, kMaxStreams);
  TL_REQUIRE(a.width > 0 && a.width <= kMaxRowFloats, "hyper: width %d outside (0, %d]", a.width, kMaxRowFloats);
  TL_REQUIRE(!a.slots || (a.slot_w && a.top > 0), "hyper: expert slots without weights");
  TL_REQUIRE(!a.table || (a.tokens && a.vocab > 0 && !a.a && !a.slots), "hyper: an embedding table without tokens, or with a sublayer's output");
  TL_REQUIRE(!a.next.w || a.h, "hyper: a norm without its output");
  size_t lds = sizeof(float) * a.width;
  if (a.route.w) {
    const RouterArgs& r = a.route;
    TL_REQUIRE(a.next.w && r.ids && r.wts && r.experts > 0 && r.top > 0 && r.top <= r.experts && !r.gate_w,
               "hyper: bad router arguments");
    TL_REQUIRE(r.kind == TL_ROUTE_TOP_LOGITS || r.kind == TL_ROUTE_SOFTMAX ||
                   (r.groups > 0 && r.experts % r.groups == 0 && r.keep > 0 && r.keep <= r.groups &&
                    (long long)r.keep * (r.experts / r.groups) >= r.top),
               "hyper: %d experts in %d groups, %d kept, top %d", r.experts, r.groups, r.keep, r.top);
    lds = sizeof(float) * (((a.width + 3) & ~3) + 2 * (size_t)r.experts + (r.groups > 0 ? r.groups : 0));
    TL_REQUIRE(lds <= 64 * 1024 - 2048, "hyper: width %d + %d experts do not fit the staged row", a.width, r.experts);
  }
  const bool v4 = (a.width & 3) == 0 && ((size_t)a.x & 15) == 0 && ((size_t)a.a & 15) == 0 && ((size_t)a.slots & 15) == 0 &&
                  ((size_t)a.sum & 15) == 0;
  if (v4) launch_hyper<4>(a, lds, s);
  else launch_hyper<1>(a, lds, s);
  TL_HIP(hipGetLastError());
  return 0;
}

extern "C" int tl_hyper_connect(float* x_dev, const float* y_dev, const float* mix_dev, const float* out_dev, float mult,
                                const float* in_dev, const float* weight_dev, const float* bias_dev, float eps, float* h_dev,
                                float* sum_dev, int num_tokens, int streams, int width, void* stream) {
  HyperArgs a = {};
  a.x = x_dev;
  a.T = num_tokens;
  a.width = width;
  a.streams = streams;
  a.a = y_dev;
  a.mix = mix_dev;
  a.out = out_dev;
  a.mult = mult;
  a.in = in_dev;
  if (in_dev) a.next = LnParams{weight_dev, bias_dev};
  a.eps = eps;
  a.h = h_dev;
  a.sum = sum_dev;
  return tl_launch_hyper(a, static_cast<hipStream_t>(stream));
}
