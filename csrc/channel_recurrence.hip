// Recurrences whose state belongs to single channels, gfx950.  Compiled without fast-math: step sizes, decays, gates and
// the recurrences are 32-bit by definition of such models.
//
//   channel_scan      S[c, n] <- exp(-exp(a_log[c, n]) d_c) S[c, n] + d_c u_c B_n ; y_c = (sum_n S[c, n] C_n + D_c u_c) *
//                     silu(gate_c), with the step size d = softplus(dt + dt_bias) per channel and token.  A workgroup owns
//                     256 / P channels of one sequence, P neighbouring lanes per channel with R states each in registers,
//                     and walks the rows in chunks staged through LDS (softplus and d * u once per value, while staging;
//                     the output gate once per value, from LDS): prompt portions and decoded rows are the same kernel
//   block_gates       a = exp(-rate * sigmoid(ra u + bias)), drive = sqrt(1 - a^2) * sigmoid(ri u + bias) * u with block-
//                     diagonal ra and ri: on the matrix cores both products of a channel meet in one wave, whose epilogue
//                     forms a and drive in fp32.  In the STEP form (every row is its sequence's only one) the epilogue
//                     also advances the state, S <- a S + drive, and writes S * gelu_tanh(gate + gate_bias)
//   gated_unit_scan   the same recurrence over prompt portions: 16 waves take 8 rows each of a 128-row chunk, scan them
//                     locally, exchange (product of a, local end state) through LDS and apply the carried state - one
//                     barrier per chunk, the next chunk's loads in flight
// 1 - a^2 is formed as -(e^(2 log a) - 1) without the cancellation a plain difference has near a = 1, and softplus keeps its
// relative precision where it is small.  Both are written here on the hardware's exponential and logarithm (one unit in the
// last place each): the library forms are three to five times the instructions, and these kernels are bound by them.
#include "common.h"
#include <math.h>
#include <type_traits>

namespace {

template <typename T> __device__ __forceinline__ float ldf(const T* p) { return (float)(*p); }
template <typename T> __device__ __forceinline__ void stf(T* p, float v) { *p = (T)v; }

template <typename F> int by_dtype(int dt, F&& f) {
  switch (dt) {
    case DT_BF16: f((bf16_t*)nullptr); return 0;
    case DT_F16: f((f16_t*)nullptr); return 0;
    case DT_F32: f((float*)nullptr); return 0;
  }
  return 1;
}

bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

// 1 - e^y for y <= 0: the Taylor polynomial up to y^8 on [-1/2, 0] (the next term is below 2^-27 of the result there), else
// the difference itself (it cannot lose more than two bits)
__device__ __forceinline__ float one_minus_exp(float y) {
  float p = 1.f + y * (1.f / 8.f);
  p = 1.f + y * (1.f / 7.f) * p;
  p = 1.f + y * (1.f / 6.f) * p;
  p = 1.f + y * (1.f / 5.f) * p;
  p = 1.f + y * (1.f / 4.f) * p;
  p = 1.f + y * (1.f / 3.f) * p;
  p = 1.f + y * (1.f / 2.f) * p;
  return y > -0.5f ? -y * p : 1.f - fast_exp(y);
}

// 0.5 (1 + tanh(y)) = sigmoid(2 y)
__device__ __forceinline__ float gelu_tanh_f(float z) {
  return z * fast_sigmoid(1.5957691216057308f * (z + 0.044715f * z * z * z));
}

// ------------------------------------------------------------------------------------------------ selective scan
struct ScanArgs {
  void* out;                                   // [T, C] of type T
  const void* u; long u_stride;                // [T, C]
  const void* dt; long dt_stride;              // [T, C] of type TD, in front of the bias and softplus
  const void* bc; long bc_stride;              // [T, >= 2 N]: [B | C]
  const void* gate; long gate_stride;          // [T, C] or null
  const float* a_log;                          // [C, N]
  const float* dt_bias; const float* d_skip;   // [C] or null
  float* state;                                // [slots, C, N]
  const int* slots; const int* qsl; const int* seq_lens;
  int C, N;
};

// grid (channel tiles, sequences), 4 waves.  Lane (channel, part): part p of a channel holds states p * R .. p * R + R - 1.
template <typename T, typename TD, int P, int R, int CH>
__global__ __launch_bounds__(256) void channel_scan_kernel(ScanArgs a) {
  constexpr int CT = 64 / P, CB = 4 * CT;      // channels per wave, per workgroup
  constexpr int NP = P * R;                    // states, padded (a padded state has B = C = 0 and stays zero)
  constexpr int NU = (CH * CB + 255) / 256, NQ = (CH * NP + 255) / 256;
  __shared__ float sd[CH][CB], sdu[CH][CB], sy[CH][CB];
  __shared__ __attribute__((aligned(16))) float sb[CH][NP], sc[CH][NP];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int part = lane & (P - 1), lc = wave * CT + lane / P;
  const int col0 = blockIdx.x * CB, s = blockIdx.y;
  const int q0 = a.qsl[s], n = a.qsl[s + 1] - q0;
  if (n <= 0) return;                          // (the whole workgroup)
  const int c = col0 + lc;
  const bool c_ok = c < a.C;
  const int cc = c_ok ? c : a.C - 1;
  const bool fresh = a.seq_lens[s] - n <= 0;   // the rows start the sequence: whatever the slot holds is not ours
  float* st = a.state + ((long)a.slots[s] * a.C + cc) * a.N + part * R;
  const float* al = a.a_log + (long)cc * a.N + part * R;
  float S[R], A2[R];
  const bool vec = R % 4 == 0 && (a.N & 3) == 0;
  if constexpr (R % 4 == 0) {
    if (vec) {
#pragma unroll
      for (int i = 0; i < R; i += 4) {
        f32x4 sv = {0.f, 0.f, 0.f, 0.f}, av = {0.f, 0.f, 0.f, 0.f};
        if (part * R + i < a.N) {
          if (!fresh) sv = *reinterpret_cast<const f32x4*>(st + i);
          av = *reinterpret_cast<const f32x4*>(al + i);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) { S[i + e] = sv[e]; A2[i + e] = av[e]; }
      }
    }
  }
  if (!vec) {
#pragma unroll
    for (int i = 0; i < R; ++i) {
      const bool ok = part * R + i < a.N;
      S[i] = ok && !fresh ? st[i] : 0.f;
      A2[i] = ok ? al[i] : 0.f;
    }
  }
  const T* up = (const T*)a.u + (long)q0 * a.u_stride + col0;
  const TD* dp = (const TD*)a.dt + (long)q0 * a.dt_stride + col0;
  const T* bp = (const T*)a.bc + (long)q0 * a.bc_stride;
  const T* gp = a.gate ? (const T*)a.gate + (long)q0 * a.gate_stride + col0 : nullptr;
  T* op = (T*)a.out + (long)q0 * a.C + col0;
  // per staged value: the channel's step bias and skip weight (channel k0 in every pass, CB divides 256)
  const int k0 = tid & (CB - 1);
  const bool k_ok = col0 + k0 < a.C;
  const int kc = k_ok ? k0 : a.C - 1 - col0;
  // A thread's share of the next chunk, raw: every load is unconditional (rows, channels and states past the end read the
  // last one there is and are not used), so nothing waits for it before it is stashed a chunk later
  T pu[NU], pz[NU], pb[NQ], pc[NQ];
  TD pd[NU];
  auto fetch = [&](int r0) {
#pragma unroll
    for (int e = 0; e < NU; ++e) {
      const long r = min(r0 + (tid + e * 256) / CB, n - 1);
      pu[e] = up[r * a.u_stride + kc];
      pd[e] = dp[r * a.dt_stride + kc];
      if (gp != nullptr) pz[e] = gp[r * a.gate_stride + kc];
    }
#pragma unroll
    for (int e = 0; e < NQ; ++e) {
      const int idx = tid + e * 256, j = min(idx & (NP - 1), a.N - 1);
      const T* row = bp + min(r0 + idx / NP, n - 1) * a.bc_stride;
      pb[e] = row[j];
      pc[e] = row[a.N + j];
    }
  };
  fetch(0);
  const float bias = a.dt_bias && k_ok ? a.dt_bias[col0 + k0] : 0.f;
  const float skip = a.d_skip && k_ok ? a.d_skip[col0 + k0] : 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i) A2[i] = -1.4426950408889634f * expf(A2[i]);
  for (int r0 = 0; r0 < n; r0 += CH) {
    float cu[NU], cz[NU];
#pragma unroll
    for (int e = 0; e < NU; ++e) {
      const int t = (tid + e * 256) / CB;
      cu[e] = (float)pu[e];
      cz[e] = gp != nullptr ? fast_silu((float)pz[e]) : 1.f;
      if (t < CH) {
        const float d = fast_softplus((float)pd[e] + bias);
        sd[t][k0] = d;
        sdu[t][k0] = d * cu[e];
      }
    }
#pragma unroll
    for (int e = 0; e < NQ; ++e) {
      const int idx = tid + e * 256, t = idx / NP, j = idx & (NP - 1);
      if (t < CH) {
        sb[t][j] = j < a.N ? (float)pb[e] : 0.f;
        sc[t][j] = j < a.N ? (float)pc[e] : 0.f;
      }
    }
    if (r0 + CH < n) fetch(r0 + CH);
    __syncthreads();
    const int rows = min(CH, n - r0);
    auto row = [&](int t) {
      const float d = sd[t][lc], du = sdu[t][lc];
      float y0 = 0.f, y1 = 0.f;                // (two chains: the sums do not wait for each other)
      if constexpr (R % 4 == 0) {
#pragma unroll
        for (int i = 0; i < R; i += 4) {
          const f32x4 bv = *reinterpret_cast<const f32x4*>(&sb[t][part * R + i]);
          const f32x4 cv = *reinterpret_cast<const f32x4*>(&sc[t][part * R + i]);
#pragma unroll
          for (int e = 0; e < 4; ++e) S[i + e] = fast_exp2(d * A2[i + e]) * S[i + e] + du * bv[e];
          y0 += S[i] * cv[0] + S[i + 2] * cv[2];
          y1 += S[i + 1] * cv[1] + S[i + 3] * cv[3];
        }
      } else {
#pragma unroll
        for (int i = 0; i < R; ++i) {
          S[i] = fast_exp2(d * A2[i]) * S[i] + du * sb[t][part * R + i];
          if (i & 1) y1 += S[i] * sc[t][part * R + i]; else y0 += S[i] * sc[t][part * R + i];
        }
      }
      const float y = parts_sum<P, true>(y0 + y1);
      if (part == 0) sy[t][lc] = y;
    };
    if (rows == CH) {
#pragma unroll (CH < 4 ? CH : 4)
      for (int t = 0; t < CH; ++t) row(t);
    } else {
      for (int t = 0; t < rows; ++t) row(t);
    }
    __syncthreads();
#pragma unroll
    for (int e = 0; e < NU; ++e) {
      const int idx = tid + e * 256, t = idx / CB;
      if (t < rows && k_ok) stf(op + (long)(r0 + t) * a.C + k0, (sy[t][k0] + skip * cu[e]) * cz[e]);
    }
  }
  if (!c_ok) return;
  if constexpr (R % 4 == 0) {
    if (vec) {
#pragma unroll
      for (int i = 0; i < R; i += 4)
        if (part * R + i < a.N) *reinterpret_cast<f32x4*>(st + i) = f32x4{S[i], S[i + 1], S[i + 2], S[i + 3]};
      return;
    }
  }
#pragma unroll
  for (int i = 0; i < R; ++i)
    if (part * R + i < a.N) st[i] = S[i];
}

// ------------------------------------------------------------------------------------------------ block-diagonal gates
struct GateArgs {
  const void* u;                               // [T, W] contiguous
  const void* ra; const void* ri;              // [blocks, n, n], out by in
  const float* ra_bias; const float* ri_bias;  // [W]
  const float* rate;                           // [W]
  float* a; float* drive;                      // [T, W] (not in the STEP form)
  void* out;                                   // [T, W] (STEP form)
  const void* gate; long gate_stride;          // [T, W] (STEP form)
  const float* gate_bias;                      // [W] or null (STEP form)
  float* state;                                // [slots, W] (STEP form)
  const int* slots; const int* seq_lens;       // (STEP form: row t is sequence t, its only row)
  int T, W, n;
};

// one channel's gates from the two products (biases already added) and its input
__device__ __forceinline__ void unit_gates(float zr, float zi, float rate, float u, float& a, float& drive) {
  const float log_a = -rate * fast_sigmoid(zr);
  a = fast_exp(log_a);
  drive = __builtin_amdgcn_sqrtf(one_minus_exp(2.0f * log_a)) * fast_sigmoid(zi) * u;
}

// any size and type: a workgroup per (row, block); a thread per output channel in turn
template <typename T>
__global__ __launch_bounds__(256) void block_gates_kernel(GateArgs p) {
  extern __shared__ float su[];
  const long t = blockIdx.x;
  const int b = blockIdx.y, n = p.n, c0 = b * n;
  const T* ur = (const T*)p.u + t * p.W + c0;
  for (int i = threadIdx.x; i < n; i += blockDim.x) su[i] = ldf(ur + i);
  __syncthreads();
  for (int o = threadIdx.x; o < n; o += blockDim.x) {
    const T* wr = (const T*)p.ra + ((long)b * n + o) * n;
    const T* wi = (const T*)p.ri + ((long)b * n + o) * n;
    float zr = 0.f, zi = 0.f;
    for (int i = 0; i < n; ++i) { zr += ldf(wr + i) * su[i]; zi += ldf(wi + i) * su[i]; }
    const int c = c0 + o;
    float a, d;
    unit_gates(zr + p.ra_bias[c], zi + p.ri_bias[c], p.rate[c], su[o], a, d);
    p.a[t * p.W + c] = a;
    p.drive[t * p.W + c] = d;
  }
}

// 16-bit types, n a multiple of 32: a wave owns 32 channels (of one block) x 16 NT rows.  Weights are the A operand, rows
// of u the B operand, so a lane ends up with 4 neighbouring channels of one row per tile.  Of the workgroup's 4 waves, WC
// lie side by side over channels and 4 / WC over rows: neighbours in either direction share fragments in the CU's cache.
template <typename T, int NT, int WC, bool STEP>
__global__ __launch_bounds__(256) void block_gates_mfma_kernel(GateArgs p) {
  using V8 = typename Vec8<T>::type;
  using V4 = typename Vec4<T>::type;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int r16 = lane & 15, g4 = lane >> 4;
  const int ct = blockIdx.x * WC + wave % WC;                    // 32-channel tile
  const int row0 = (blockIdx.y * (4 / WC) + wave / WC) * 16 * NT;
  if (ct * 32 >= p.W || row0 >= p.T) return;                     // (no barrier below: a wave may leave)
  const int n = p.n, b = ct * 32 / n, o0 = ct * 32 - b * n;      // (n % 32 == 0: a tile lies in one block)
  const T* wr = (const T*)p.ra + ((long)b * n + o0 + r16) * n + 8 * g4;
  const T* wi = (const T*)p.ri + ((long)b * n + o0 + r16) * n + 8 * g4;
  const T* up[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) up[t] = (const T*)p.u + (long)min(row0 + 16 * t + r16, p.T - 1) * p.W + b * n + 8 * g4;
  f32x4 zr[2][NT], zi[2][NT];
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int t = 0; t < NT; ++t) zr[m][t] = zi[m][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
  for (int k = 0; k < n; k += 32) {
    V8 fr[2], fi[2], fu[NT];
#pragma unroll
    for (int m = 0; m < 2; ++m) { fr[m] = ld8<T>(wr + (long)16 * m * n + k); fi[m] = ld8<T>(wi + (long)16 * m * n + k); }
#pragma unroll
    for (int t = 0; t < NT; ++t) fu[t] = ld8<T>(up[t] + k);
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        zr[m][t] = mfma16(fr[m], fu[t], zr[m][t]);
        zi[m][t] = mfma16(fi[m], fu[t], zi[m][t]);
      }
  }
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    const int c = ct * 32 + 16 * m + 4 * g4;
    const f32x4 br = *reinterpret_cast<const f32x4*>(p.ra_bias + c), bi = *reinterpret_cast<const f32x4*>(p.ri_bias + c);
    const f32x4 rt = *reinterpret_cast<const f32x4*>(p.rate + c);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int row = row0 + 16 * t + r16;
      if (row >= p.T) continue;
      const V4 uv = *reinterpret_cast<const V4*>((const T*)p.u + (long)row * p.W + c);
      f32x4 av, dv;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float a, d;
        unit_gates(zr[m][t][e] + br[e], zi[m][t][e] + bi[e], rt[e], (float)uv[e], a, d);
        av[e] = a;
        dv[e] = d;
      }
      if constexpr (STEP) {
        float* st = p.state + (long)p.slots[row] * p.W + c;
        f32x4 S = dv;
        if (p.seq_lens[row] > 1) S = av * *reinterpret_cast<const f32x4*>(st) + dv;
        *reinterpret_cast<f32x4*>(st) = S;
        const V4 gv = *reinterpret_cast<const V4*>((const T*)p.gate + (long)row * p.gate_stride + c);
        V4 o;
#pragma unroll
        for (int e = 0; e < 4; ++e)
          o[e] = (T)(S[e] * gelu_tanh_f((float)gv[e] + (p.gate_bias ? p.gate_bias[c + e] : 0.f)));
        *reinterpret_cast<V4*>((T*)p.out + (long)row * p.W + c) = o;
      } else {
        *reinterpret_cast<f32x4*>(p.a + (long)row * p.W + c) = av;
        *reinterpret_cast<f32x4*>(p.drive + (long)row * p.W + c) = dv;
      }
    }
  }
}

// ------------------------------------------------------------------------------------------------ first-order scan
// grid (tiles of 64 channels, sequences), NW waves; wave w takes rows w * L .. w * L + L - 1 of every chunk of NW * L.
template <typename T, int NW, int L>
__global__ __launch_bounds__(64 * NW) void gated_unit_scan_kernel(T* __restrict__ out, const float* __restrict__ a,
                                                                  const float* __restrict__ drive,
                                                                  const T* __restrict__ gate, long gate_stride,
                                                                  const float* __restrict__ gate_bias,
                                                                  float* __restrict__ state, const int* __restrict__ slots,
                                                                  const int* __restrict__ qsl,
                                                                  const int* __restrict__ seq_lens, int W) {
  __shared__ float sp[2][NW][64], sq[2][NW][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int c = blockIdx.x * 64 + lane, s = blockIdx.y;
  const int q0 = qsl[s], n = qsl[s + 1] - q0;
  if (n <= 0) return;                                            // (the whole workgroup)
  const bool ok = c < W;
  const int cc = ok ? c : W - 1;
  const float* ap = a + (long)q0 * W + cc;
  const float* dp = drive + (long)q0 * W + cc;
  const T* gp = gate + (long)q0 * gate_stride + cc;
  T* op = out + (long)q0 * W + cc;
  const float gb = gate_bias ? gate_bias[cc] : 0.f;
  float* st = state + (long)slots[s] * W + cc;
  float S = seq_lens[s] - n > 0 ? *st : 0.f;                     // the state in front of the chunk, in every wave
  float na[L], nd[L];
  T ng[L];
  auto fetch = [&](int r0) {                                     // (rows past the end read the last one: no load is conditional)
#pragma unroll
    for (int i = 0; i < L; ++i) {
      const long r = min(r0 + wave * L + i, n - 1);
      na[i] = ap[r * W];
      nd[i] = dp[r * W];
      ng[i] = gp[r * gate_stride];
    }
  };
  fetch(0);
  int buf = 0;
  for (int r0 = 0; r0 < n; r0 += NW * L, buf ^= 1) {
    float va[L], vd[L], vg[L];
    float P = 1.f, Q = 0.f;
#pragma unroll
    for (int i = 0; i < L; ++i) {
      const bool live = r0 + wave * L + i < n;
      va[i] = live ? na[i] : 1.f;                                // (rows past the end leave the state as it is)
      vd[i] = live ? nd[i] : 0.f;
      P *= va[i];
      Q = va[i] * Q + vd[i];
      vg[i] = gelu_tanh_f((float)ng[i] + gb);
    }
    if (r0 + NW * L < n) fetch(r0 + NW * L);
    if constexpr (NW > 1) {
      sp[buf][wave][lane] = P;
      sq[buf][wave][lane] = Q;
      __syncthreads();         // (the other buffer is free again: every wave has read it before it came here)
    }
    float carry = S;
    if constexpr (NW > 1) {
      float run = S;
#pragma unroll
      for (int w = 0; w < NW; ++w) {
        if (w == wave) carry = run;
        run = sp[buf][w][lane] * run + sq[buf][w][lane];
      }
      S = run;
    } else {
      S = P * S + Q;
    }
#pragma unroll
    for (int i = 0; i < L; ++i) {
      carry = va[i] * carry + vd[i];
      const int r = r0 + wave * L + i;
      if (r < n && ok) stf(op + (long)r * W, carry * vg[i]);
    }
  }
  if (wave == 0 && ok) *st = S;
}

}  // namespace

// u [T, u_stride], bc [T, bc_stride] = [B (N) | C (N)], gate [T, gate_stride] (or null) and out [T, C] of type dtype; dt
// [T, dt_stride] of type dt_dtype (dtype or fp32); a_log [C, N], dt_bias [C] / d_skip [C] fp32 or null; state fp32
// [slots, C, N], 16-byte aligned; N <= 256.  max_rows: the most rows any sequence brings (0 = unknown)
VDAMD_API int vdamd_channel_scan(void* out, const void* u, long u_stride, const void* dt, long dt_stride, const void* bc,
                                 long bc_stride, const void* gate, long gate_stride, const float* a_log,
                                 const float* dt_bias, const float* d_skip, float* state, const int* slots,
                                 const int* qsl, const int* seq_lens, int num_seqs, int C, int N, int max_rows, int dtype,
                                 int dt_dtype, hipStream_t stream) {
  if (num_seqs <= 0) return 0;
  if (C <= 0 || N <= 0 || N > 256 || (dt_dtype != DT_F32 && dt_dtype != dtype)) return 1;
  if (!aligned16(state) || !aligned16(a_log)) return 1;
  ScanArgs a{out, u, u_stride, dt, dt_stride, bc, bc_stride, gate, gate_stride, a_log, dt_bias, d_skip, state, slots, qsl,
             seq_lens, C, N};
  const bool step = max_rows == 1;
  // lanes per channel: as few as hold the states four by four; more where the launch would leave a compute unit fewer than two workgroups
  int parts = N <= 16 ? 4 : (N <= 32 ? 8 : 16);
  if (!step)
    while (parts < 16 && (long)num_seqs * ((C + 256 / parts - 1) / (256 / parts)) < 512) parts <<= 1;
  const int r = (N + parts - 1) / parts;
  const dim3 grid((C + 256 / parts - 1) / (256 / parts), num_seqs);
  const int rc = by_dtype(dtype, [&](auto* tp) {
    using TT = std::remove_pointer_t<decltype(tp)>;
#define CSCAN(TD_, P_, R_, CH_) hipLaunchKernelGGL((channel_scan_kernel<TT, TD_, P_, R_, CH_>), grid, dim3(256), 0, stream, a)
#define CSCAN_D(P_, R_)                                                      \
  do {                                                                       \
    if (dt_dtype == DT_F32) {                                                \
      if (step) CSCAN(float, P_, R_, 1); else CSCAN(float, P_, R_, 16);      \
    } else {                                                                 \
      if (step) CSCAN(TT, P_, R_, 1); else CSCAN(TT, P_, R_, 16);            \
    }                                                                        \
  } while (0)
    if (parts == 4) CSCAN_D(4, 4);
    else if (parts == 8) { if (r <= 2) CSCAN_D(8, 2); else CSCAN_D(8, 4); }
    else {
      if (r <= 1) CSCAN_D(16, 1);
      else if (r <= 2) CSCAN_D(16, 2);
      else if (r <= 4) CSCAN_D(16, 4);
      else if (r <= 8) CSCAN_D(16, 8);
      else CSCAN_D(16, 16);
    }
#undef CSCAN_D
#undef CSCAN
  });
  if (rc) return 1;
  HIP_LAUNCH_CHECK();
  return 0;
}

// Whether block_gates / gated_unit_step run on the matrix cores for this type and block size.
VDAMD_API int vdamd_block_gates_mfma_ok(int n, int dtype) { return dtype != DT_F32 && n % 32 == 0 ? 1 : 0; }

// u [T, W] contiguous, ra / ri [blocks, n, n] of type dtype (16-byte aligned), biases and rate fp32 [W]; W % n == 0.  With
// state null: a and drive fp32 [T, W].  Else the STEP form (matrix-core sizes only): row t is the only row of sequence t,
// the state fp32 [slots, W] moves on and out [T, W] = S * gelu_tanh(gate [T, gate_stride] + gate_bias).
VDAMD_API int vdamd_block_gates(float* a, float* drive, const void* u, const void* ra, const float* ra_bias,
                                const void* ri, const float* ri_bias, const float* rate, void* out, const void* gate,
                                long gate_stride, const float* gate_bias, float* state, const int* slots,
                                const int* seq_lens, int T, int W, int n, int dtype, hipStream_t stream) {
  if (T <= 0) return 0;
  if (W <= 0 || n <= 0 || W % n) return 1;
  const bool step = state != nullptr;
  if (step ? (out == nullptr || gate == nullptr || slots == nullptr || seq_lens == nullptr) : (a == nullptr || drive == nullptr))
    return 1;
  GateArgs p{u, ra, ri, ra_bias, ri_bias, rate, a, drive, out, gate, gate_stride, gate_bias, state, slots, seq_lens, T, W, n};
  const bool mfma = vdamd_block_gates_mfma_ok(n, dtype) && aligned16(u) && aligned16(ra) && aligned16(ri) &&
                    aligned16(ra_bias) && aligned16(ri_bias) && aligned16(rate) && aligned16(a) && aligned16(drive) &&
                    aligned16(state) && aligned16(out) && (reinterpret_cast<uintptr_t>(gate) & 7) == 0 && gate_stride % 4 == 0;
  if (step && !mfma) return 1;
  const int rc = by_dtype(dtype, [&](auto* tp) {
    using TT = std::remove_pointer_t<decltype(tp)>;
    if constexpr (!std::is_same_v<TT, float>) {
      if (mfma) {
        // four row tiles per wave and two by two waves where that leaves every compute unit two workgroups, else one
        const bool tall = (long)((W / 32 + 1) / 2) * ((T + 127) / 128) >= 512;
        const dim3 grid = tall ? dim3((W / 32 + 1) / 2, (T + 127) / 128) : dim3((W / 32 + 3) / 4, (T + 15) / 16);
        if (step && tall) hipLaunchKernelGGL((block_gates_mfma_kernel<TT, 4, 2, true>), grid, dim3(256), 0, stream, p);
        else if (step) hipLaunchKernelGGL((block_gates_mfma_kernel<TT, 1, 4, true>), grid, dim3(256), 0, stream, p);
        else if (tall) hipLaunchKernelGGL((block_gates_mfma_kernel<TT, 4, 2, false>), grid, dim3(256), 0, stream, p);
        else hipLaunchKernelGGL((block_gates_mfma_kernel<TT, 1, 4, false>), grid, dim3(256), 0, stream, p);
        return;
      }
    }
    hipLaunchKernelGGL((block_gates_kernel<TT>), dim3(T, W / n), dim3(n >= 256 ? 256 : (n >= 128 ? 128 : 64)),
                       (size_t)n * sizeof(float), stream, p);
  });
  if (rc) return 1;
  HIP_LAUNCH_CHECK();
  return 0;
}

// a, drive fp32 [T, W]; gate [T, gate_stride] and out [T, W] of type dtype; state fp32 [slots, W].  max_rows: the most rows
// any sequence brings (0 = unknown)
VDAMD_API int vdamd_gated_unit_scan(void* out, const float* a, const float* drive, const void* gate, long gate_stride,
                                    const float* gate_bias, float* state, const int* slots, const int* qsl,
                                    const int* seq_lens, int num_seqs, int W, int max_rows, int dtype,
                                    hipStream_t stream) {
  if (num_seqs <= 0) return 0;
  if (W <= 0) return 1;
  const dim3 grid((W + 63) / 64, num_seqs);
  const int rc = by_dtype(dtype, [&](auto* tp) {
    using TT = std::remove_pointer_t<decltype(tp)>;
#define GUS(NW_, L_)                                                                                                   \
  hipLaunchKernelGGL((gated_unit_scan_kernel<TT, NW_, L_>), grid, dim3(64 * NW_), 0, stream, (TT*)out, a, drive,       \
                     (const TT*)gate, gate_stride, gate_bias, state, slots, qsl, seq_lens, W)
    if (max_rows > 0 && max_rows <= 4) GUS(1, 1);
    else GUS(16, 8);
#undef GUS
  });
  if (rc) return 1;
  HIP_LAUNCH_CHECK();
  return 0;
}
