// tl_ssm.hip — selective state space with one decay per head and token (Mamba-2's form), a mixer of a layer-list model: per head
// a state S [state][vdim] instead of a cache of keys; the heads of a group share B and C. Per token and head
//
//     dt = softplus(dt_raw + dt_bias);   S <- exp(-exp(A_log) dt) S + dt B x^T;   y = S^T C + D x;   y <- y silu(z)
//
// x, B, C have passed a causal convolution + bias + silu (tl_conv.hip). Everything here is FP32: products on the FP32 matrix
// instruction, decays as exp of log-decay sums that are accumulated in double (two neighbouring sums may be large and close).
//
// Several tokens are walked in blocks of 64. Inside a block, with c_i the inclusive sum of the log-decays -exp(A_log) dt,
//
//     Y_i = sum_{j <= i} exp(c_i - c_j) dt_j (C_i . B_j) x_j  +  exp(c_i) C_i S_before  (+ D x_i),
//     S_after = exp(c_last) S_before + sum_j exp(c_last - c_j) dt_j B_j x_j^T:
//
// the recurrence becomes three small matrix products per block; only S is handed on from block to block.
//   ssm_gram    C_i . B_j of every block and GROUP (lower triangle of 64 x 64): heads / groups heads share it.
//   ssm_walk    one workgroup of 4 waves per (32 value channels, head) walks the blocks in order. S lives in accumulator
//               registers: wave w holds the state rows 32 (w + 4 k) .. + 31 of its 32 columns, in the layout in which the matrix
//               instruction leaves a result -- which is also the operand layout its product with C needs (the order of a sum's
//               terms is free as long as both operands agree), so S never moves. The waves' partial Y meet in LDS.
//   ssm_step    one token: a workgroup per (32 value channels, head) forms the convolution of the channels it needs itself
//               (history read, not written: other workgroups read it too), updates its piece of S and reads it out.
//   part_norm   RMS norm of a row in equal parts, in place; for one token it also shifts the convolution's history, whose
//               readers are done by then.
#include <math.h>

#include "tl_bf16.h"
#include "tl_stack.h"

namespace {

typedef float ssm_f32x4 __attribute__((ext_vector_type(4)));
typedef float ssm_f32x16 __attribute__((ext_vector_type(16)));

constexpr int SSM_Q = 64;                 // tokens of a block
constexpr int SSM_LD = 36, SSM_PLD = 68;  // padded LDS rows of 32 / 64 floats (16-byte pieces, spread over the banks)

__device__ __forceinline__ float ssm_softplus(float z) { return z > 20.0f ? z : log1pf(expf(z)); }
__device__ __forceinline__ float ssm_silu(float z) { return z / (1.0f + expf(-z)); }
// row of a 32 x 32 result held in accumulator register e of lane half h
__device__ __forceinline__ int ssm_row(int e, int h) { return (e & 3) + 8 * (e >> 2) + 4 * h; }

// four neighbouring floats p[d .. d + 3] of a row of n values (zeros beyond); vec: 16-byte loads are possible
__device__ __forceinline__ ssm_f32x4 ssm_ld4(const float* p, int d, int n, bool vec) {
  if (vec && d + 4 <= n) return *reinterpret_cast<const ssm_f32x4*>(p + d);
  ssm_f32x4 v;
#pragma unroll
  for (int c = 0; c < 4; ++c) v[c] = d + c < n ? p[d + c] : 0.0f;
  return v;
}

// grid (blocks, groups), 3 waves: the tiles (0,0), (1,0), (1,1) of the block's 64 x 64 products
__global__ __launch_bounds__(192) void ssm_gram_kernel(const SsmScanArgs a, int vec) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 31, h = lane >> 5;
  const int ti = wave == 0 ? 0 : 1, tj = wave == 2 ? 1 : 0;
  const int t0 = blockIdx.x * SSM_Q, g = blockIdx.y;
  if (ti == 1 && t0 + 32 >= a.T) return;  // no token of the second half: nothing reads those tiles
  const int N = a.state_n, inner = a.heads * a.vdim;
  auto row = [&](int t) { return t < a.T ? t : a.T - 1; };  // rows beyond the call carry weight 0 where they are used
  const float* bp = a.xbc + (size_t)row(t0 + tj * 32 + r) * a.ld + inner + (size_t)g * N;
  const float* cp = a.xbc + (size_t)row(t0 + ti * 32 + r) * a.ld + inner + (size_t)(a.groups + g) * N;
  ssm_f32x16 acc;
#pragma unroll
  for (int e = 0; e < 16; ++e) acc[e] = 0.0f;
  for (int d = 0; d < N; d += 8) {
    const ssm_f32x4 cv = ssm_ld4(cp, d + 4 * h, N, vec), bv = ssm_ld4(bp, d + 4 * h, N, vec);
#pragma unroll
    for (int c = 0; c < 4; ++c) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(cv[c], bv[c], acc, 0, 0, 0);
  }
  float* o = a.gram + ((size_t)blockIdx.x * a.groups + g) * SSM_Q * SSM_Q;
#pragma unroll
  for (int e = 0; e < 16; ++e) o[(size_t)(ti * 32 + ssm_row(e, h)) * SSM_Q + tj * 32 + r] = acc[e];
}

struct SsmLds {  // dynamic LDS of ssm_walk_kernel
  double cum[SSM_Q];                 // c_i
  float p[SSM_Q][SSM_PLD];           // exp(c_i - c_j) dt_j (C_i . B_j), j <= i
  float x[SSM_Q][SSM_LD];            // x of the block
  float part[4][SSM_Q][SSM_LD];      // the waves' partial Y
  float dt[SSM_Q], w[SSM_Q], e[SSM_Q];  // dt_j; exp(c_last - c_j) dt_j; exp(c_i)
};

// NT state tiles of 32 rows per wave: state <= 128 NT
template <int NT>
__global__ __launch_bounds__(256, 2) void ssm_walk_kernel(const SsmScanArgs a, int vec) {
  extern __shared__ __attribute__((aligned(16))) unsigned char ssm_lds_raw[];
  SsmLds& L = *reinterpret_cast<SsmLds*>(ssm_lds_raw);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r = lane & 31, h = lane >> 5;
  const int v0 = blockIdx.x * 32, head = blockIdx.y, g = head / (a.heads / a.groups);
  const int N = a.state_n, vdim = a.vdim, inner = a.heads * vdim;
  const bool vlive = v0 + r < vdim;
  const float* xp = a.xbc + (size_t)head * vdim + v0;
  const float* bp = a.xbc + inner + (size_t)g * N;
  const float* cp = bp + (size_t)a.groups * N;
  const float rate = expf(a.a_log[head]), dtb = a.dt_bias[head], dskip = a.d[head];
  float* sp = a.state + (size_t)head * N * vdim + v0;
  ssm_f32x16 S[NT];
#pragma unroll
  for (int k = 0; k < NT; ++k)
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int n = 32 * (wave + 4 * k) + ssm_row(e, h);
      S[k][e] = n < N && vlive ? sp[(size_t)n * vdim + r] : 0.0f;
    }
  for (int t0 = 0; t0 < a.T; t0 += SSM_Q) {
    const int nt = a.T - t0 < SSM_Q ? a.T - t0 : SSM_Q;
    const bool two = nt > 32;  // tokens in the second half of the block
    auto row = [&](int t) { return (size_t)(t0 + (t < nt ? t : nt - 1)); };
    if (wave == 0) {
      const float dt = lane < nt ? ssm_softplus(a.dt_raw[(size_t)(t0 + lane) * a.dt_ld + head] + dtb) : 0.0f;
      double c = -(double)(rate * dt);
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const double up = __shfl_up(c, o);
        if (lane >= o) c += up;
      }
      const double tot = __shfl(c, 63);
      L.cum[lane] = c;
      L.dt[lane] = dt;
      L.w[lane] = dt * expf((float)(tot - c));
      L.e[lane] = expf((float)c);
    }
#pragma unroll
    for (int i = 0; i < SSM_Q * 32 / 256; ++i) {
      const int idx = i * 256 + tid, t = idx >> 5, c = idx & 31;
      L.x[t][c] = t < nt && v0 + c < vdim ? xp[(size_t)(t0 + t) * a.ld + c] : 0.0f;
    }
    // C S of the waves' state rows: the scores of the first product's operand come straight from the token's own row
    ssm_f32x16 acc[2];
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[tt][e] = 0.0f;
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) {
      if (tt == 1 && !two) break;
      const float* cr = cp + row(tt * 32 + r) * a.ld;
#pragma unroll
      for (int k = 0; k < NT; ++k) {
        const int n0 = 32 * (wave + 4 * k);
        if (n0 >= N) break;
        ssm_f32x4 cv[4];
#pragma unroll
        for (int q = 0; q < 4; ++q) cv[q] = ssm_ld4(cr, n0 + 8 * q + 4 * h, N, vec);
#pragma unroll
        for (int q = 0; q < 4; ++q)
#pragma unroll
          for (int c = 0; c < 4; ++c) acc[tt] = __builtin_amdgcn_mfma_f32_32x32x2f32(cv[q][c], S[k][4 * q + c], acc[tt], 0, 0, 0);
      }
    }
    __syncthreads();  // dt, c_i and x of the block are in LDS
    const float* gp = a.gram + ((size_t)(t0 / SSM_Q) * a.groups + g) * SSM_Q * SSM_Q;
#pragma unroll
    for (int i = 0; i < SSM_Q * SSM_Q / 256; ++i) {
      const int idx = i * 256 + tid, ti = idx >> 6, tj = idx & 63;
      float v = 0.0f;
      if (tj <= ti && ti < nt) v = gp[idx] * expf((float)(L.cum[ti] - L.cum[tj])) * L.dt[tj];
      L.p[ti][tj] = v;
    }
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[tt][e] *= L.e[tt * 32 + ssm_row(e, h)];
    __syncthreads();  // P is whole
    // P X: the first half's tokens look at 32 columns (8 a wave), the second half's at 64 (16 a wave)
    {
      const int j0 = 8 * wave + 4 * h;
      const ssm_f32x4 pv = *reinterpret_cast<const ssm_f32x4*>(&L.p[r][j0]);
#pragma unroll
      for (int c = 0; c < 4; ++c) acc[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(pv[c], L.x[j0 + c][r], acc[0], 0, 0, 0);
      if (two) {
#pragma unroll
        for (int q = 0; q < 2; ++q) {
          const int j1 = 16 * wave + 8 * q + 4 * h;
          const ssm_f32x4 pw = *reinterpret_cast<const ssm_f32x4*>(&L.p[32 + r][j1]);
#pragma unroll
          for (int c = 0; c < 4; ++c) acc[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(pw[c], L.x[j1 + c][r], acc[1], 0, 0, 0);
        }
      }
    }
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int e = 0; e < 16; ++e) L.part[wave][tt * 32 + ssm_row(e, h)][r] = acc[tt][e];
    // S <- exp(c_last) S + B^T (w x)
    const float decay = L.e[SSM_Q - 1];
#pragma unroll
    for (int k = 0; k < NT; ++k) {
      const int n = 32 * (wave + 4 * k) + r;
      if (32 * (wave + 4 * k) >= N) break;
#pragma unroll
      for (int e = 0; e < 16; ++e) S[k][e] *= decay;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        if (half == 1 && !two) break;
        float bv[16];
#pragma unroll
        for (int s = 0; s < 16; ++s) bv[s] = n < N ? bp[row(32 * half + 2 * s + h) * a.ld + n] : 0.0f;
#pragma unroll
        for (int s = 0; s < 16; ++s) {
          const int j = 32 * half + 2 * s + h;
          S[k] = __builtin_amdgcn_mfma_f32_32x32x2f32(bv[s], L.w[j] * L.x[j][r], S[k], 0, 0, 0);
        }
      }
    }
    __syncthreads();  // the partial Y are whole
#pragma unroll
    for (int i = 0; i < SSM_Q * 32 / 256; ++i) {
      const int idx = i * 256 + tid, t = idx >> 5, c = idx & 31;
      if (t >= nt || v0 + c >= vdim) continue;
      float y = ((L.part[0][t][c] + L.part[1][t][c]) + (L.part[2][t][c] + L.part[3][t][c])) + dskip * L.x[t][c];
      if (a.z) y *= ssm_silu(a.z[(size_t)(t0 + t) * a.z_ld + (size_t)head * vdim + v0 + c]);
      a.y[(size_t)(t0 + t) * inner + (size_t)head * vdim + v0 + c] = y;
    }
    __syncthreads();  // x and the partial Y may be overwritten
  }
#pragma unroll
  for (int k = 0; k < NT; ++k)
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int n = 32 * (wave + 4 * k) + ssm_row(e, h);
      if (n < N && vlive) sp[(size_t)n * vdim + r] = S[k][e];
    }
}

// grid (value channels in 32s, heads), 256 threads: 8 column quads x 32 state rows, the state in passes of 32 rows
__global__ __launch_bounds__(256) void ssm_step_kernel(const SsmStepArgs a, int vec) {
  extern __shared__ __attribute__((aligned(16))) float sl[];  // B [N] | C [N] | x [32]
  __shared__ float red[4][32];
  const int tid = threadIdx.x, cq = tid & 7, rg = tid >> 3;
  const int v0 = blockIdx.x * 32, head = blockIdx.y, g = head / (a.heads / a.groups);
  const int N = a.state_n, vdim = a.vdim, inner = a.heads * vdim, H = a.taps - 1, CH = inner + 2 * a.groups * N;
  float* sB = sl;
  float* sC = sl + N;
  float* sx = sl + 2 * N;
  float* sp = a.state + (size_t)head * N * vdim + v0 + 4 * cq;
  const int left = vdim - v0 - 4 * cq;  // columns of this thread's quad that exist (<= 0: none)
  constexpr int PF = 4;                 // passes whose state is asked for before the convolution
  float4 st[PF];
  auto load = [&](int n) __attribute__((always_inline)) {
    float4 v = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (n < N && left > 0) {
      const float* p = sp + (size_t)n * vdim;
      if (vec) return *reinterpret_cast<const float4*>(p);
      v.x = p[0];
      if (left > 1) v.y = p[1];
      if (left > 2) v.z = p[2];
      if (left > 3) v.w = p[3];
    }
    return v;
  };
#pragma unroll
  for (int i = 0; i < PF; ++i) st[i] = load(rg + 32 * i);
  const float dt = ssm_softplus(a.p[inner + CH + head] + a.dt_bias[head]);
  const float decay = expf(-expf(a.a_log[head]) * dt);
  const int nx = vdim - v0 < 32 ? vdim - v0 : 32;
  for (int i = tid; i < nx + 2 * N; i += 256) {  // the channels this workgroup needs: its x columns, the group's B and C
    const int c = i < nx ? head * vdim + v0 + i : i < nx + N ? inner + g * N + (i - nx) : inner + (a.groups + g) * N + (i - nx - N);
    const unsigned short* w = a.conv + (size_t)c * a.taps;
    float u = 0.0f;
    for (int j = 0; j < H; ++j) u += tl_bf2f(w[j]) * a.hist[(size_t)j * CH + c];
    u += tl_bf2f(w[H]) * a.p[inner + c];
    u = ssm_silu(u + a.conv_b[c]);
    if (i < nx) sx[i] = u;
    else sB[i - nx] = u;  // (C lies behind B)
  }
  __syncthreads();
  float4 xv = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  if (left > 0) xv.x = dt * sx[4 * cq];
  if (left > 1) xv.y = dt * sx[4 * cq + 1];
  if (left > 2) xv.z = dt * sx[4 * cq + 2];
  if (left > 3) xv.w = dt * sx[4 * cq + 3];
  float4 y = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  for (int n0 = 0; n0 < N; n0 += 32 * PF) {
    if (n0 > 0) {
#pragma unroll
      for (int i = 0; i < PF; ++i) st[i] = load(n0 + rg + 32 * i);
    }
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int n = n0 + rg + 32 * i;
      if (n >= N || left <= 0) continue;
      const float b = sB[n], c = sC[n];
      float4 s = st[i];
      s.x = decay * s.x + b * xv.x;
      s.y = decay * s.y + b * xv.y;
      s.z = decay * s.z + b * xv.z;
      s.w = decay * s.w + b * xv.w;
      y.x += c * s.x;
      y.y += c * s.y;
      y.z += c * s.z;
      y.w += c * s.w;
      float* p = sp + (size_t)n * vdim;
      if (vec) {
        *reinterpret_cast<float4*>(p) = s;
      } else {
        p[0] = s.x;
        if (left > 1) p[1] = s.y;
        if (left > 2) p[2] = s.z;
        if (left > 3) p[3] = s.w;
      }
    }
  }
#pragma unroll
  for (int o = 8; o < 64; o <<= 1) {  // the eight state rows a wave works on side by side
    y.x += __shfl_xor(y.x, o);
    y.y += __shfl_xor(y.y, o);
    y.z += __shfl_xor(y.z, o);
    y.w += __shfl_xor(y.w, o);
  }
  if ((tid & 63) < 8) {
    float* o = &red[tid >> 6][4 * cq];
    o[0] = y.x, o[1] = y.y, o[2] = y.z, o[3] = y.w;
  }
  __syncthreads();
  if (tid < nx) {
    const float v = ((red[0][tid] + red[1][tid]) + (red[2][tid] + red[3][tid])) + a.d[head] * sx[tid];
    a.y[(size_t)head * vdim + v0 + tid] = v * ssm_silu(a.p[(size_t)head * vdim + v0 + tid]);
  }
}

// grid (T * parts (+ the history's channels in 256s)), 256 threads a part
__global__ __launch_bounds__(256) void part_norm_kernel(const PartNormArgs a) {
  __shared__ float red[4];
  const int tid = threadIdx.x, units = a.T * a.parts;
  if ((int)blockIdx.x >= units) {
    const int c = ((int)blockIdx.x - units) * 256 + tid, H = a.taps - 1;
    if (c >= a.channels) return;
    for (int j = 0; j + 1 < H; ++j) a.hist[(size_t)j * a.channels + c] = a.hist[(size_t)(j + 1) * a.channels + c];
    a.hist[(size_t)(H - 1) * a.channels + c] = a.hist_in[c];
    return;
  }
  const int t = blockIdx.x / a.parts, part = blockIdx.x - t * a.parts, n = a.width / a.parts;
  float* x = a.x + (size_t)t * a.width + (size_t)part * n;
  const float* w = a.w + (size_t)part * n;
  float ss = 0.0f;
  for (int c = tid; c < n; c += 256) ss += x[c] * x[c];
  ss = tl_wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float inv = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)n + a.eps);
  for (int c = tid; c < n; c += 256) x[c] = x[c] * inv * w[c];
}

template <int NT>
int launch_walk(const SsmScanArgs& a, int vec, hipStream_t s) {
  static TlDeviceOnce lds_raised;  // per instantiation, per device
  TL_TRY(tl_raise_lds_limit(ssm_walk_kernel<NT>, 160 * 1024, lds_raised));
  ssm_walk_kernel<NT><<<dim3((a.vdim + 31) / 32, a.heads), 256, sizeof(SsmLds), s>>>(a, vec);
  TL_HIP(hipGetLastError());
  return 0;
}

}  // namespace

size_t tl_ssm_gram_floats(int T, int groups) { return (size_t)((T + SSM_Q - 1) / SSM_Q) * groups * SSM_Q * SSM_Q; }

int tl_launch_ssm_scan(const SsmScanArgs& a, hipStream_t s) {
  TL_REQUIRE(a.xbc && a.dt_raw && a.dt_bias && a.a_log && a.d && a.state && a.y && a.gram && a.T > 0, "ssm_scan: bad arguments");
  TL_REQUIRE(a.heads > 0 && a.heads <= 65535 && a.groups > 0 && a.groups <= 65535 && a.heads % a.groups == 0 && a.vdim > 0,
             "ssm_scan: %d heads in %d groups, value size %d", a.heads, a.groups, a.vdim);
  TL_REQUIRE(a.state_n > 0 && a.state_n <= 512, "ssm_scan: state size %d outside (0, 512]", a.state_n);
  TL_REQUIRE(a.ld >= a.heads * a.vdim + 2 * a.groups * a.state_n && a.dt_ld >= a.heads && (!a.z || a.z_ld >= a.heads * a.vdim),
             "ssm_scan: row strides %d / %d / %d", a.ld, a.dt_ld, a.z_ld);
  // 16-byte pieces of B and C rows
  const int vec = (a.state_n & 3) == 0 && (a.ld & 3) == 0 && ((a.heads * a.vdim) & 3) == 0 && ((size_t)a.xbc & 15) == 0;
  ssm_gram_kernel<<<dim3((a.T + SSM_Q - 1) / SSM_Q, a.groups), 192, 0, s>>>(a, vec);
  const int nt = (a.state_n + 127) / 128;
  if (nt <= 1) return launch_walk<1>(a, vec, s);
  if (nt <= 2) return launch_walk<2>(a, vec, s);
  return launch_walk<4>(a, vec, s);
}

int tl_launch_ssm_step(const SsmStepArgs& a, hipStream_t s) {
  TL_REQUIRE(a.p && a.conv && a.conv_b && a.dt_bias && a.a_log && a.d && a.state && a.y, "ssm_step: bad arguments");
  TL_REQUIRE(a.heads > 0 && a.heads <= 65535 && a.groups > 0 && a.heads % a.groups == 0 && a.vdim > 0 && a.state_n > 0 &&
                 a.state_n <= 4096,
             "ssm_step: %d heads in %d groups, sizes %d / %d", a.heads, a.groups, a.state_n, a.vdim);
  TL_REQUIRE(a.taps >= 1 && (a.taps == 1 || a.hist), "ssm_step: %d taps", a.taps);
  const int vec = (a.vdim & 3) == 0 && ((size_t)a.state & 15) == 0;
  ssm_step_kernel<<<dim3((a.vdim + 31) / 32, a.heads), 256, sizeof(float) * (2 * (size_t)a.state_n + 32), s>>>(a, vec);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_part_norm(const PartNormArgs& a, hipStream_t s) {
  TL_REQUIRE(a.x && a.w && a.T > 0 && a.parts > 0 && a.width > 0 && a.width % a.parts == 0, "part_norm: %d channels in %d parts",
             a.width, a.parts);
  TL_REQUIRE(!a.hist || (a.T == 1 && a.hist_in && a.taps > 1 && a.channels > 0), "part_norm: a history rides along for one token");
  const long long blocks = (long long)a.T * a.parts + (a.hist ? (a.channels + 255) / 256 : 0);
  TL_REQUIRE(blocks <= 0x7fffffffLL, "part_norm: launch too large");
  part_norm_kernel<<<(unsigned)blocks, 256, 0, s>>>(a);
  TL_HIP(hipGetLastError());
  return 0;
}

extern "C" int tl_state_space(const float* xbc_dev, int ld, const float* dt_raw_dev, int dt_ld, const float* dt_bias_dev,
                              const float* a_log_dev, const float* d_dev, const float* z_dev, int z_ld, float* state_dev,
                              float* y_dev, int num_tokens, int heads, int groups, int state, int vdim, void* stream) {
  TL_REQUIRE(num_tokens > 0 && groups > 0, "tl_state_space: bad arguments");
  SsmScanArgs a = {};
  a.xbc = xbc_dev;
  a.ld = ld;
  a.dt_raw = dt_raw_dev;
  a.dt_ld = dt_ld;
  a.dt_bias = dt_bias_dev;
  a.a_log = a_log_dev;
  a.d = d_dev;
  a.z = z_dev;
  a.z_ld = z_ld;
  a.state = state_dev;
  a.y = y_dev;
  a.T = num_tokens;
  a.heads = heads;
  a.groups = groups;
  a.state_n = state;
  a.vdim = vdim;
  void* ws = nullptr;
  TL_TRY(tl_scratch(TL_SCRATCH_SSM, sizeof(float) * tl_ssm_gram_floats(num_tokens, groups), &ws));
  a.gram = static_cast<float*>(ws);
  return tl_launch_ssm_scan(a, static_cast<hipStream_t>(stream));
}

extern "C" int tl_state_space_step(const float* p_dev, const void* conv_bf16_dev, const float* conv_bias_dev, int taps,
                                   const float* history_dev, const float* dt_bias_dev, const float* a_log_dev, const float* d_dev,
                                   float* state_dev, float* y_dev, int heads, int groups, int state, int vdim, void* stream) {
  SsmStepArgs a = {};
  a.p = p_dev;
  a.conv = static_cast<const uint16_t*>(conv_bf16_dev);
  a.conv_b = conv_bias_dev;
  a.taps = taps;
  a.hist = history_dev;
  a.dt_bias = dt_bias_dev;
  a.a_log = a_log_dev;
  a.d = d_dev;
  a.state = state_dev;
  a.y = y_dev;
  a.heads = heads;
  a.groups = groups;
  a.state_n = state;
  a.vdim = vdim;
  return tl_launch_ssm_step(a, static_cast<hipStream_t>(stream));
}

extern "C" int tl_part_norm(float* x_dev, const float* weight_dev, int num_tokens, int width, int parts, float eps,
                            float* history_dev, const float* in_dev, int taps, int channels, void* stream) {
  PartNormArgs a = {};
  a.x = x_dev;
  a.w = weight_dev;
  a.T = num_tokens;
  a.width = width;
  a.parts = parts;
  a.eps = eps;
  a.hist = history_dev;
  a.hist_in = in_dev;
  a.taps = taps;
  a.channels = channels;
  return tl_launch_part_norm(a, static_cast<hipStream_t>(stream));
}
