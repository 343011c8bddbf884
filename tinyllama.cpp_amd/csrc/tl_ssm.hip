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
//   ssm_gram    C_i . B_j of every block and GROUP (lower triangle of 64 x 64): heads / groups heads share it; and, per block and
//               head, dt, c and the two exponentials that depend on one token only.
//   ssm_walk    one workgroup of 4 waves per (32 value channels, head) walks the blocks in order. S lives in accumulator
//               registers: wave w holds the state rows 32 (w + 4 k) .. + 31 of its 32 columns, in the layout in which the matrix
//               instruction leaves a result -- which is also the operand layout its product with C needs (the order of a sum's
//               terms is free as long as both operands agree), so S never moves. The waves' partial Y meet in LDS.
//   ssm_step    one token: a workgroup per (32 value channels, head) forms the convolution of the channels it needs itself
//               (history read, not written: other workgroups read it too), updates its piece of S and reads it out.
//   With log_decay the same walk is linear attention with one CONSTANT decay per head, S <- decay S + k v^T, o = S^T q: x = v, B = k,
//   C = q, dt = 1, no skip (lightning_step: its one-token form).
//   part_norm   RMS norm of a row in equal parts, in place, optionally times a sigmoid gate; for one token it also shifts the convolution's history, whose
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
// the same from the hardware's exp2 and reciprocal: relative error near 1e-7 |z| where the result matters
__device__ __forceinline__ float ssm_silu_fast(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }
// base (the same for the wave) + a lane's own element: one 32-bit offset register per load
__device__ __forceinline__ float ssm_at(const float* base, unsigned e) {
  return *reinterpret_cast<const float*>(reinterpret_cast<const char*>(base) + (size_t)(e * 4u));
}
__device__ __forceinline__ ssm_f32x4 ssm_at4(const float* base, unsigned e) {
  return *reinterpret_cast<const ssm_f32x4*>(reinterpret_cast<const char*>(base) + (size_t)(e * 4u));
}
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

// What the walk needs of a block of tokens and a head besides x, B, C, and what it keeps in LDS of it
struct SsmSteps {
  double cum[SSM_Q];                    // c_i
  float dt[SSM_Q], w[SSM_Q], e[SSM_Q];  // dt_j; exp(c_last - c_j) dt_j; exp(c_i)
};
constexpr int SSM_STEP_FLOATS = sizeof(SsmSteps) / sizeof(float);
static_assert(SSM_STEP_FLOATS == 256 + 64, "ssm_walk_kernel copies 256 + 64 floats");

// grid (blocks, groups + heads in threes), 3 waves. blockIdx.y < groups: the tiles (0,0), (1,0), (1,1) of the block's 64 x 64
// products of that group; otherwise a wave per head: its SsmSteps
__global__ __launch_bounds__(192) void ssm_gram_kernel(const SsmScanArgs a, int vec) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r = lane & 31, h = lane >> 5;
  const int t0 = blockIdx.x * SSM_Q, g = blockIdx.y;
  float* grams = a.gram;
  SsmSteps* steps = reinterpret_cast<SsmSteps*>(a.gram + (size_t)gridDim.x * a.groups * SSM_Q * SSM_Q);
  if (g >= a.groups) {
    const int head = (g - a.groups) * 3 + wave;
    if (head >= a.heads) return;
    const bool in = t0 + lane < a.T;
    const float dt = !in ? 0.0f : a.log_decay ? 1.0f : ssm_softplus(a.dt_raw[(size_t)(t0 + lane) * a.dt_ld + head] + a.dt_bias[head]);
    double c = !in ? 0.0 : a.log_decay ? a.log_decay[head] : -(double)(expf(a.a_log[head]) * dt);
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double up = __shfl_up(c, o);
      if (lane >= o) c += up;
    }
    const double tot = __shfl(c, 63);
    SsmSteps* o = steps + (size_t)blockIdx.x * a.heads + head;
    o->cum[lane] = c;
    o->dt[lane] = dt;
    o->w[lane] = dt * expf((float)(tot - c));
    o->e[lane] = expf((float)c);
    return;
  }
  const int ti = wave == 0 ? 0 : 1, tj = wave == 2 ? 1 : 0;
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
  float* o = grams + ((size_t)blockIdx.x * a.groups + g) * SSM_Q * SSM_Q;
#pragma unroll
  for (int e = 0; e < 16; ++e) o[(size_t)(ti * 32 + ssm_row(e, h)) * SSM_Q + tj * 32 + r] = acc[e];
}

struct SsmLds {  // dynamic LDS of ssm_walk_kernel; what a block's last readers may still read while the next one arrives is doubled
  SsmSteps st[2];
  float x[2][SSM_Q][SSM_LD];         // x of the block
  float p[SSM_Q][SSM_PLD];           // exp(c_i - c_j) dt_j (C_i . B_j), j <= i
  float part[4][SSM_Q][SSM_LD];      // the waves' partial Y
};

// NT state tiles of 32 rows per wave: state <= 128 NT. Whatever comes from memory for a block is asked for while the block before
// is worked on (B and C only with NT == 1: registers), since a workgroup is often alone on its CU.
// EVEN: state and vdim are multiples of 32, the tokens whole blocks, and B, C rows can be read in 16-byte pieces.
template <int NT, bool EVEN>
__global__ __launch_bounds__(256, NT == 1 ? 2 : 1) void ssm_walk_kernel(const SsmScanArgs a, int vec) {
  extern __shared__ __attribute__((aligned(16))) unsigned char ssm_lds_raw[];
  SsmLds& L = *reinterpret_cast<SsmLds*>(ssm_lds_raw);
  constexpr bool PF = NT == 1;
  const int tid = threadIdx.x, lane = tid & 63, r = lane & 31, h = lane >> 5;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int v0 = blockIdx.x * 32, head = blockIdx.y, g = head / (a.heads / a.groups);
  const int N = a.state_n, vdim = a.vdim, inner = a.heads * vdim, last = a.T - 1;
  const int blocks = (a.T + SSM_Q - 1) / SSM_Q;
  const bool vlive = EVEN || v0 + r < vdim;
  const float* xp = a.xbc + (size_t)head * vdim;
  const float* bp = a.xbc + inner + (size_t)g * N;
  const float* cp = bp + (size_t)a.groups * N;
  const float* zp = a.z ? a.z + (size_t)head * vdim : nullptr;
  const float dskip = a.d ? a.d[head] : 0.0f;
  const float* stp = a.gram + (size_t)blocks * a.groups * SSM_Q * SSM_Q + (size_t)head * SSM_STEP_FLOATS;
  float* sp = a.state + (size_t)head * N * vdim + v0;
  // (row offsets fit 32 bits: the launcher checks; rows beyond the call repeat its last row and carry weight 0)
  auto row = [&](int t) __attribute__((always_inline)) { return (unsigned)(t < last ? t : last); };
  // this thread's elements of a block: x and z (token i * 8 + tid / 32, column tid % 32), the products (row i * 4 + tid / 64)
  const int xt = tid >> 5, xc = tid & 31;
  const bool xlive = EVEN || v0 + xc < vdim;
  const unsigned xv = xlive ? v0 + xc : vdim - 1;  // (a column beyond vdim repeats the last one and is not stored)
  float xr[8], zr[8], gr[16], sr[2];
  // a block that the call fills: a pointer per row that the wave shares, one offset per lane for the whole kernel
  const unsigned ld = a.ld, zld = a.z_ld;
  const unsigned xo = xt * ld + xv, zo = xt * zld + xv;
  auto rows8 = [&](const float* p, unsigned stride, unsigned off, int b, float* to) __attribute__((always_inline)) {
    if (EVEN) {
      const float* q = p + (size_t)b * SSM_Q * stride;
#pragma unroll
      for (int i = 0; i < 8; ++i) to[i] = ssm_at(q + (size_t)(8 * i) * stride, off);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) to[i] = ssm_at(p, row(b * SSM_Q + i * 8 + xt) * stride + xv);
    }
  };
  auto fetch_x = [&](int b) __attribute__((always_inline)) {
    rows8(xp, ld, xo, b, xr);
    const float* s = stp + (size_t)b * a.heads * SSM_STEP_FLOATS;
    sr[0] = ssm_at(s, tid);
    sr[1] = ssm_at(s, 256 + (tid & 63));
  };
  auto fetch_z = [&](int b) __attribute__((always_inline)) {
    if (zp) rows8(zp, zld, zo, b, zr);
  };
  auto fetch_g = [&](int b) __attribute__((always_inline)) {
    const float* gp = a.gram + ((size_t)b * a.groups + g) * SSM_Q * SSM_Q;
#pragma unroll
    for (int i = 0; i < 16; ++i) gr[i] = ssm_at(gp + i * 256, tid);  // (never-written tiles are not used below)
  };
  ssm_f32x4 cr[PF ? 2 : 1][4];
  auto fetch_c = [&](int b, int tt, int k, ssm_f32x4* to) __attribute__((always_inline)) {
    const int n0 = 32 * (wave + 4 * k);
    if (EVEN) {
      const float* c = cp + (size_t)(b * SSM_Q + tt * 32) * ld + n0;
#pragma unroll
      for (int q = 0; q < 4; ++q) to[q] = ssm_at4(c + 8 * q, r * ld + 4 * h);
    } else {
      const float* c = cp + (size_t)row(b * SSM_Q + tt * 32 + r) * ld;
#pragma unroll
      for (int q = 0; q < 4; ++q) to[q] = ssm_ld4(c, n0 + 8 * q + 4 * h, N, vec);
    }
  };
  float br[PF ? 2 : 1][16];
  auto fetch_b = [&](int b, int half, int k, float* to) __attribute__((always_inline)) {
    const int n = 32 * (wave + 4 * k) + r;
    const unsigned nn = EVEN || n < N ? n : N - 1;  // (rows beyond the state meet zeros of C and are not stored)
    if (EVEN) {
      const float* p = bp + (size_t)(b * SSM_Q + 32 * half) * ld;
#pragma unroll
      for (int s = 0; s < 16; ++s) to[s] = ssm_at(p + (size_t)(2 * s) * ld, h * ld + nn);
    } else {
#pragma unroll
      for (int s = 0; s < 16; ++s) to[s] = ssm_at(bp, row(b * SSM_Q + 32 * half + 2 * s + h) * ld + nn);
    }
  };
  const bool mine = 32 * wave < N;  // this wave holds state rows at all
  ssm_f32x16 S[NT];
#pragma unroll
  for (int k = 0; k < NT; ++k)
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int n = 32 * (wave + 4 * k) + ssm_row(e, h);
      S[k][e] = n < N && vlive ? sp[(size_t)n * vdim + r] : 0.0f;
    }
  fetch_x(0);
  fetch_g(0);
  if (PF && mine) {
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) fetch_c(0, tt, 0, cr[PF ? tt : 0]);
#pragma unroll
    for (int tt = 0; tt < 2; ++tt) fetch_b(0, tt, 0, br[PF ? tt : 0]);
  }
  fetch_z(0);
  for (int b = 0; b < blocks; ++b) {
    const int nb = b + 1 < blocks ? b + 1 : b;  // (after the last block its own values are read once more: no branch)
    const int t0 = b * SSM_Q, nt = EVEN || a.T - t0 > SSM_Q ? SSM_Q : a.T - t0;
    const bool two = EVEN || nt > 32;  // tokens in the second half of the block
    SsmSteps& st = L.st[b & 1];
    float (*x)[SSM_LD] = L.x[b & 1];
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i * 8 + xt][xc] = EVEN || t0 + i * 8 + xt < a.T ? xr[i] : 0.0f;
    reinterpret_cast<float*>(&st)[tid] = sr[0];
    reinterpret_cast<float*>(&st)[256 + (tid & 63)] = sr[1];  // (four writers of one value)
    __syncthreads();  // x and the steps of the block are in LDS
    fetch_x(nb);
    // C S over this wave's state rows
    ssm_f32x16 acc[2];
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[tt][e] = 0.0f;
    if (PF) {
      if (mine) {
#pragma unroll
        for (int q = 0; q < 4; ++q)
#pragma unroll
          for (int c = 0; c < 4; ++c)
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
              acc[tt] = __builtin_amdgcn_mfma_f32_32x32x2f32(cr[PF ? tt : 0][q][c], S[0][4 * q + c], acc[tt], 0, 0, 0);
#pragma unroll
        for (int tt = 0; tt < 2; ++tt) fetch_c(nb, tt, 0, cr[PF ? tt : 0]);
      }
    } else {
#pragma unroll
      for (int tt = 0; tt < 2; ++tt) {
        if (tt == 1 && !two) continue;
#pragma unroll
        for (int k = 0; k < NT; ++k) {
          if (32 * (wave + 4 * k) >= N) continue;
          fetch_c(b, tt, k, cr[0]);
#pragma unroll
          for (int q = 0; q < 4; ++q)
#pragma unroll
            for (int c = 0; c < 4; ++c)
              acc[tt] = __builtin_amdgcn_mfma_f32_32x32x2f32(cr[0][q][c], S[k][4 * q + c], acc[tt], 0, 0, 0);
        }
      }
    }
    {
      const int tj = lane;  // (this thread's column of the products in every row it fills)
      const double cj = st.cum[tj];
      const float dj = st.dt[tj];
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int ti = i * 4 + wave;
        const float d = fminf((float)(st.cum[ti] - cj), 0.0f);
        const float v = gr[i] * __expf(d) * dj;  // (hardware exp2: its error is 1e-7 of the largest weight, 1)
        L.p[ti][tj] = tj <= ti && ti < nt ? v : 0.0f;
      }
    }
    fetch_g(nb);
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[tt][e] *= st.e[tt * 32 + ssm_row(e, h)];
    __syncthreads();  // P is whole
    // P X: the first half's tokens look at 32 columns (8 a wave), the second half's at 64 (16 a wave)
    {
      const int j0 = 8 * wave + 4 * h;
      const ssm_f32x4 pv = *reinterpret_cast<const ssm_f32x4*>(&L.p[r][j0]);
#pragma unroll
      for (int c = 0; c < 4; ++c) acc[0] = __builtin_amdgcn_mfma_f32_32x32x2f32(pv[c], x[j0 + c][r], acc[0], 0, 0, 0);
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        const int j1 = 16 * wave + 8 * q + 4 * h;
        const ssm_f32x4 pw = *reinterpret_cast<const ssm_f32x4*>(&L.p[32 + r][j1]);
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[1] = __builtin_amdgcn_mfma_f32_32x32x2f32(pw[c], x[j1 + c][r], acc[1], 0, 0, 0);
      }
    }
    // S <- exp(c_last) S + B^T (w x)
    const float decay = st.e[SSM_Q - 1];
#pragma unroll
    for (int k = 0; k < NT; ++k) {
      if (32 * (wave + 4 * k) >= N) continue;
#pragma unroll
      for (int e = 0; e < 16; ++e) S[k][e] *= decay;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        if (half == 1 && !two) continue;
        float* bv = br[PF ? half : 0];
        if (!PF) fetch_b(b, half, k, bv);
        float xw[16];
#pragma unroll
        for (int s = 0; s < 16; ++s) xw[s] = st.w[32 * half + 2 * s + h] * x[32 * half + 2 * s + h][r];
#pragma unroll
        for (int s = 0; s < 16; ++s) S[k] = __builtin_amdgcn_mfma_f32_32x32x2f32(bv[s], xw[s], S[k], 0, 0, 0);
        if (PF) fetch_b(nb, half, 0, bv);
      }
    }
#pragma unroll
    for (int tt = 0; tt < 2; ++tt)
#pragma unroll
      for (int e = 0; e < 16; ++e) L.part[wave][tt * 32 + ssm_row(e, h)][r] = acc[tt][e];
    __syncthreads();  // the partial Y are whole
    float y[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int t = i * 8 + xt;
      y[i] = ((L.part[0][t][xc] + L.part[1][t][xc]) + (L.part[2][t][xc] + L.part[3][t][xc])) + dskip * x[t][xc];
    }
    if (zp) {
#pragma unroll
      for (int i = 0; i < 8; ++i) y[i] *= ssm_silu_fast(zr[i]);
    }
    float* yp = a.y + (size_t)t0 * inner + (size_t)head * vdim + v0;
    if (EVEN) {
#pragma unroll
      for (int i = 0; i < 8; ++i) yp[(size_t)(8 * i + xt) * inner + xc] = y[i];
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (i * 8 + xt < nt && xlive) yp[(size_t)(8 * i + xt) * inner + xc] = y[i];
    }
    fetch_z(nb);
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

// grid (T * parts (+ the history's channels in blockDim.x s)), a workgroup a part: 256 threads, or 1024 where a launch is a few long
// rows and nothing but round trips to memory
__global__ __launch_bounds__(1024) void part_norm_kernel(const PartNormArgs a) {
  __shared__ float red[16];
  const int tid = threadIdx.x, units = a.T * a.parts, step = blockDim.x;
  if ((int)blockIdx.x >= units) {
    const int c = ((int)blockIdx.x - units) * step + tid, H = a.taps - 1;
    if (c >= a.channels) return;
    for (int j = 0; j + 1 < H; ++j) a.hist[(size_t)j * a.channels + c] = a.hist[(size_t)(j + 1) * a.channels + c];
    a.hist[(size_t)(H - 1) * a.channels + c] = a.hist_in[c];
    return;
  }
  const int t = blockIdx.x / a.parts, part = blockIdx.x - t * a.parts, n = a.width / a.parts;
  float* x = a.x + (size_t)t * a.width + (size_t)part * n;
  const float* w = a.w + (size_t)part * n;
  float ss = 0.0f;
  for (int c = tid; c < n; c += step) ss += x[c] * x[c];
  ss = tl_wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  ss = 0.0f;
  for (int w = 0; w < step >> 6; ++w) ss += red[w];
  const float inv = 1.0f / sqrtf(ss / (float)n + a.eps);
  const float* gt = a.gate ? a.gate + (size_t)t * a.gate_ld + (size_t)part * n : nullptr;
  for (int c = tid; c < n; c += step) x[c] = x[c] * inv * w[c] * (gt ? 1.0f / (1.0f + expf(-gt[c])) : 1.0f);
}

// grid (value channels in 32s, heads), 256 threads: 8 column quads x 32 state rows, the state in passes of 32 rows
__global__ __launch_bounds__(256) void lightning_step_kernel(const LightningStepArgs a, int vec) {
  extern __shared__ __attribute__((aligned(16))) float sl[];  // k [dim] | q [dim]
  __shared__ float red[4][32];
  const int tid = threadIdx.x, cq = tid & 7, rg = tid >> 3;
  const int v0 = blockIdx.x * 32, head = blockIdx.y, N = a.dim, vdim = a.vdim;
  const float* vp = a.vkq + (size_t)head * vdim + v0 + 4 * cq;
  const float* kp = a.vkq + (size_t)a.heads * vdim + (size_t)head * N;
  const float* qp = kp + (size_t)a.heads * N;
  float* sp = a.state + (size_t)head * N * vdim + v0 + 4 * cq;
  const int left = vdim - v0 - 4 * cq;  // columns of this thread's quad that exist (<= 0: none)
  auto load4 = [&](const float* p, bool wide) __attribute__((always_inline)) {
    float4 v = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (left <= 0) return v;
    if (wide) return *reinterpret_cast<const float4*>(p);
    v.x = p[0];
    if (left > 1) v.y = p[1];
    if (left > 2) v.z = p[2];
    if (left > 3) v.w = p[3];
    return v;
  };
  constexpr int PF = 4;  // passes whose state is in flight together
  const float4 v4 = load4(vp, false);
  const float decay = (float)exp(a.log_decay[head]);
  for (int i = tid; i < N; i += 256) {
    sl[i] = kp[i];
    sl[N + i] = qp[i];
  }
  float4 y = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
  for (int n0 = 0; n0 < N; n0 += 32 * PF) {
    float4 st[PF];
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int n = n0 + rg + 32 * i;
      st[i] = n < N ? load4(sp + (size_t)n * vdim, vec != 0) : make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    }
    if (n0 == 0) __syncthreads();
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int n = n0 + rg + 32 * i;
      if (n >= N || left <= 0) continue;
      const float k = sl[n], q = sl[N + n];
      float4 s = st[i];
      s.x = decay * s.x + k * v4.x;
      s.y = decay * s.y + k * v4.y;
      s.z = decay * s.z + k * v4.z;
      s.w = decay * s.w + k * v4.w;
      y.x += q * s.x;
      y.y += q * s.y;
      y.z += q * s.z;
      y.w += q * s.w;
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
  if (tid < 32 && v0 + tid < vdim)
    a.y[(size_t)head * vdim + v0 + tid] = (red[0][tid] + red[1][tid]) + (red[2][tid] + red[3][tid]);
}

template <int NT, bool EVEN>
int launch_walk(const SsmScanArgs& a, int vec, hipStream_t s) {
  static TlDeviceOnce lds_raised;  // per instantiation, per device
  auto kernel = ssm_walk_kernel<NT, EVEN>;
  TL_TRY(tl_raise_lds_limit(kernel, 160 * 1024, lds_raised));
  kernel<<<dim3((a.vdim + 31) / 32, a.heads), 256, sizeof(SsmLds), s>>>(a, vec);
  TL_HIP(hipGetLastError());
  return 0;
}

}  // namespace

size_t tl_ssm_gram_floats(int T, int heads, int groups) {
  return (size_t)((T + SSM_Q - 1) / SSM_Q) * ((size_t)groups * SSM_Q * SSM_Q + (size_t)heads * SSM_STEP_FLOATS);
}

int tl_launch_ssm_scan(const SsmScanArgs& a, hipStream_t s) {
  TL_REQUIRE(a.xbc && (a.log_decay || (a.dt_raw && a.dt_bias && a.a_log && a.d)) && a.state && a.y && a.gram && a.T > 0,
             "ssm_scan: bad arguments");
  TL_REQUIRE(a.heads > 0 && a.heads <= 65535 && a.groups > 0 && a.groups <= 65535 && a.heads % a.groups == 0 && a.vdim > 0,
             "ssm_scan: %d heads in %d groups, value size %d", a.heads, a.groups, a.vdim);
  TL_REQUIRE(a.state_n > 0 && a.state_n <= 512, "ssm_scan: state size %d outside (0, 512]", a.state_n);
  TL_REQUIRE(a.ld >= a.heads * a.vdim + 2 * a.groups * a.state_n && (a.log_decay || a.dt_ld >= a.heads) && (!a.z || a.z_ld >= a.heads * a.vdim),
             "ssm_scan: row strides %d / %d / %d", a.ld, a.dt_ld, a.z_ld);
  // 16-byte pieces of B and C rows
  const int vec = (a.state_n & 3) == 0 && (a.ld & 3) == 0 && ((a.heads * a.vdim) & 3) == 0 && ((size_t)a.xbc & 15) == 0;
  TL_REQUIRE(a.T < (1 << 30) / (a.ld > a.z_ld ? a.ld : a.z_ld), "ssm_scan: %d tokens in rows of %d / %d", a.T, a.ld, a.z_ld);
  TL_REQUIRE(((size_t)a.gram & 7) == 0, "ssm_scan: scratch not aligned");
  const bool even = vec && (a.state_n & 31) == 0 && (a.vdim & 31) == 0;
  if (even && a.T > SSM_Q && a.T % SSM_Q) {  // whole blocks on the even kernel, the rest as a call of its own
    SsmScanArgs w = a, rest = a;
    w.T = a.T - a.T % SSM_Q;
    rest.T = a.T - w.T;
    rest.xbc += (size_t)w.T * a.ld;
    if (a.dt_raw) rest.dt_raw += (size_t)w.T * a.dt_ld;
    if (a.z) rest.z += (size_t)w.T * a.z_ld;
    rest.y += (size_t)w.T * a.heads * a.vdim;
    TL_TRY(tl_launch_ssm_scan(w, s));
    return tl_launch_ssm_scan(rest, s);
  }
  ssm_gram_kernel<<<dim3((a.T + SSM_Q - 1) / SSM_Q, a.groups + (a.heads + 2) / 3), 192, 0, s>>>(a, vec);
  const bool fast = even && a.T % SSM_Q == 0;
  const int nt = (a.state_n + 127) / 128;
  if (nt <= 1) return fast ? launch_walk<1, true>(a, vec, s) : launch_walk<1, false>(a, vec, s);
  if (nt <= 2) return fast ? launch_walk<2, true>(a, vec, s) : launch_walk<2, false>(a, vec, s);
  return fast ? launch_walk<4, true>(a, vec, s) : launch_walk<4, false>(a, vec, s);
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

int tl_launch_lightning_step(const LightningStepArgs& a, hipStream_t s) {
  TL_REQUIRE(a.vkq && a.log_decay && a.state && a.y && a.heads > 0 && a.heads <= 65535 && a.dim > 0 && a.dim <= 4096 && a.vdim > 0,
             "lightning_step: bad arguments");
  const int vec = (a.vdim & 3) == 0 && ((size_t)a.state & 15) == 0;
  lightning_step_kernel<<<dim3((a.vdim + 31) / 32, a.heads), 256, sizeof(float) * 2 * (size_t)a.dim, s>>>(a, vec);
  TL_HIP(hipGetLastError());
  return 0;
}

int tl_launch_part_norm(const PartNormArgs& a, hipStream_t s) {
  TL_REQUIRE(a.x && a.w && a.T > 0 && a.parts > 0 && a.width > 0 && a.width % a.parts == 0, "part_norm: %d channels in %d parts",
             a.width, a.parts);
  TL_REQUIRE(!a.gate || a.gate_ld >= a.width, "part_norm: gate rows of %d for %d channels", a.gate_ld, a.width);
  TL_REQUIRE(!a.hist || (a.T == 1 && a.hist_in && a.taps > 1 && a.channels > 0), "part_norm: a history rides along for one token");
  const int th = (long long)a.T * a.parts <= 64 && a.width / a.parts >= 1024 ? 1024 : 256;
  const long long blocks = (long long)a.T * a.parts + (a.hist ? (a.channels + th - 1) / th : 0);
  TL_REQUIRE(blocks <= 0x7fffffffLL, "part_norm: launch too large");
  part_norm_kernel<<<(unsigned)blocks, th, 0, s>>>(a);
  TL_HIP(hipGetLastError());
  return 0;
}

extern "C" int tl_state_space(const float* xbc_dev, int ld, const float* dt_raw_dev, int dt_ld, const float* dt_bias_dev,
                              const float* a_log_dev, const float* d_dev, const float* z_dev, int z_ld, float* state_dev,
                              float* y_dev, int num_tokens, int heads, int groups, int state, int vdim, void* stream) {
  TL_REQUIRE(num_tokens > 0 && groups > 0 && heads > 0, "tl_state_space: bad arguments");
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
  TL_TRY(tl_scratch(TL_SCRATCH_SSM, sizeof(float) * tl_ssm_gram_floats(num_tokens, heads, groups), &ws));
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

extern "C" int tl_constant_decay_attention(const float* vkq_dev, int ld, const double* log_decay_dev, float* state_dev, float* o_dev,
                                           int num_tokens, int heads, int dim, int vdim, void* stream) {
  TL_REQUIRE(num_tokens > 0 && heads > 0 && dim > 0 && vdim > 0, "tl_constant_decay_attention: bad arguments");
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (num_tokens == 1) return tl_launch_lightning_step(LightningStepArgs{vkq_dev, log_decay_dev, state_dev, o_dev, heads, dim, vdim}, s);
  SsmScanArgs a = {};
  a.xbc = vkq_dev;
  a.ld = ld;
  a.log_decay = log_decay_dev;
  a.state = state_dev;
  a.y = o_dev;
  a.T = num_tokens;
  a.heads = a.groups = heads;
  a.state_n = dim;
  a.vdim = vdim;
  void* ws = nullptr;
  TL_TRY(tl_scratch(TL_SCRATCH_SSM, sizeof(float) * tl_ssm_gram_floats(num_tokens, heads, heads), &ws));
  a.gram = static_cast<float*>(ws);
  return tl_launch_ssm_scan(a, s);
}

extern "C" int tl_gated_row_norm(float* x_dev, const float* weight_dev, const float* gate_dev, int gate_ld, int num_tokens, int width,
                                 float eps, void* stream) {
  PartNormArgs a = {};
  a.x = x_dev;
  a.w = weight_dev;
  a.T = num_tokens;
  a.width = width;
  a.parts = 1;
  a.eps = eps;
  a.gate = gate_dev;
  a.gate_ld = gate_ld;
  return tl_launch_part_norm(a, static_cast<hipStream_t>(stream));
}
