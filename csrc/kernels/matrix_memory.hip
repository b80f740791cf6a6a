// Matrix memory with exponential gates over the engine's per-sequence state slots.  Per (sequence, head), all fp32:
//
//   i = cap tanh((z_i + b_i) / cap),  f = logsigmoid(cap tanh((z_f + b_f) / cap))
//   m' = max(f + m, i)                               running maximum, 0 before the first token
//   S  = e^(f + m - m') S + e^(i - m') k v^T         [D, V]
//   n  = e^(f + m - m') n + e^(i - m') k             [D]
//   o  = S^T q / (max(|n . q|, e^-m') + den_eps)
//   out = o / rms(o) * norm_w * sigmoid(gate) * out_scale       per head, in the element type
//
// Walk (any sizes, both element types): one workgroup per (sequence, head) does everything of a token in one pass.  A
// thread owns 4 neighbouring columns of every RG-th row of S; with few enough rows per thread the state stays in
// registers between the tokens, otherwise it streams through memory.  A decode step is one token: the launch is the
// state's traffic, read and written once in 16-byte pieces.
#include "api_memory.h"
#include "common.h"

namespace dsse {
namespace {

constexpr int kWalkThreads = 512;

DEV float softcap_f(float z, float cap) { return cap * tanhf(z / cap); }
DEV float logsigmoid_f(float x) { return fminf(x, 0.0f) - log1pf(expf(-fabsf(x))); }
DEV float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }

template <int VEC>
DEV void ld_vec(const float* p, float (&v)[VEC]) {
  if constexpr (VEC == 4) {
    const f32x4 t = ld_global<f32x4>(p);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = t[e];
  } else {
    v[0] = *p;
  }
}
template <int VEC>
DEV void st_vec(float* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4) *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  else p[0] = v[0];
}

// NR: rows of S a thread keeps in registers (every row of its share), 0: the state streams through memory per token
template <typename T, int VEC, int NR>
__global__ __launch_bounds__(kWalkThreads) void matrix_memory_walk_kernel(MatrixMemoryParams p) {
  extern __shared__ __align__(16) float lds[];
  const int h = blockIdx.x, seq = blockIdx.y;
  const int ql = p.q_len[seq];
  if (ql <= 0) return;
  const int D = p.D, V = p.V, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  constexpr int kWaves = kWalkThreads / 64;
  const int CG = V / VEC, RG = kWalkThreads / CG;  // column groups, row groups
  const int rg = tid / CG, c0 = (tid - rg * CG) * VEC;
  const bool on = rg < RG;
  float* qs = lds;            // [D] query times its scale
  float* ks = qs + D;         // [D]
  float* red = ks + D;        // [RG][V] partial read-outs
  float* sum1 = red + RG * V; // [kWaves]
  float* sum2 = sum1 + kWaves;
  const int row0 = p.q_start[seq];
  const bool fresh = p.ctx_len[seq] - ql == 0;
  const int64_t entry = (int64_t)p.state_slot[seq] * p.H + h;
  float* st = p.state + entry * D * V;
  float* nm = p.norm + entry * (D + 1);
  float S[NR > 0 ? NR : 1][VEC];
  if constexpr (NR > 0) {
#pragma unroll
    for (int j = 0; j < NR; ++j) {
      const int d = rg + j * RG;
#pragma unroll
      for (int e = 0; e < VEC; ++e) S[j][e] = 0.0f;
      if (on && d < D && !fresh) ld_vec<VEC>(st + (int64_t)d * V + c0, S[j]);
    }
  }
  float n = tid < D && !fresh ? nm[tid] : 0.0f;
  float m = fresh ? 0.0f : nm[D];
  for (int t = 0; t < ql; ++t) {
    const int64_t row = row0 + t;
    const float* z = p.gates + row * p.ldz;
    const float ig = softcap_f(z[h] + p.gate_b[h], p.cap);
    const float fg = logsigmoid_f(softcap_f(z[p.H + h] + p.gate_b[p.H + h], p.cap));
    float k = 0.f, q = 0.f;
    if (tid < D) {
      k = p.k[row * p.ldk + h * D + tid];
      q = p.q[row * p.ldq + h * D + tid] * p.q_scale;
      ks[tid] = k;
      qs[tid] = q;
    }
    float v[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] = on ? p.v[row * p.ldv + h * V + c0 + e] : 0.0f;
    const float mn = fmaxf(fg + m, ig);
    const float keep = expf(fg + m - mn), put = expf(ig - mn);
    m = mn;
#pragma unroll
    for (int e = 0; e < VEC; ++e) v[e] *= put;
    n = keep * n + put * k;
    const float part = wave_sum(n * q);
    if (lane == 0) sum1[wave] = part;
    __syncthreads();  // q, k and the normaliser's partial products are staged
    float o[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) o[e] = 0.0f;
    if (on) {
      if constexpr (NR > 0) {
#pragma unroll
        for (int j = 0; j < NR; ++j) {
          const int d = rg + j * RG;
          const float kd = d < D ? ks[d] : 0.0f, qd = d < D ? qs[d] : 0.0f;
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            S[j][e] = keep * S[j][e] + kd * v[e];
            o[e] += S[j][e] * qd;
          }
        }
      } else {
        const bool zero = fresh && t == 0;
        for (int d = rg; d < D; d += RG) {
          float s[VEC];
          float* sp = st + (int64_t)d * V + c0;
#pragma unroll
          for (int e = 0; e < VEC; ++e) s[e] = 0.0f;
          if (!zero) ld_vec<VEC>(sp, s);
#pragma unroll
          for (int e = 0; e < VEC; ++e) {
            s[e] = keep * s[e] + ks[d] * v[e];
            o[e] += s[e] * qs[d];
          }
          st_vec<VEC>(sp, s);
        }
      }
#pragma unroll
      for (int e = 0; e < VEC; ++e) red[rg * V + c0 + e] = o[e];
    }
    float nq = 0.f;
#pragma unroll
    for (int w = 0; w < kWaves; ++w) nq += sum1[w];
    const float den = fmaxf(fabsf(nq), expf(-m)) + p.den_eps;
    __syncthreads();  // the partial read-outs are complete; sum1, q and k have been read
    float y = 0.f;
    if (tid < V) {
      for (int r = 0; r < RG; ++r) y += red[r * V + tid];
      y /= den;
    }
    const float ss = wave_sum(y * y);
    if (lane == 0) sum2[wave] = ss;
    __syncthreads();
    if (tid < V) {
      float tot = 0.f;
#pragma unroll
      for (int w = 0; w < kWaves; ++w) tot += sum2[w];
      const float inv = 1.0f / sqrtf(tot / (float)V + p.eps);
      const float g = sigmoid_f(p.out_gate[row * p.ldg + h * V + tid]);
      reinterpret_cast<T*>(p.out)[row * p.ldo + h * V + tid] = (T)(y * inv * p.norm_w[h * V + tid] * g * p.out_scale);
    }
  }
  if constexpr (NR > 0) {
#pragma unroll
    for (int j = 0; j < NR; ++j) {
      const int d = rg + j * RG;
      if (on && d < D) st_vec<VEC>(st + (int64_t)d * V + c0, S[j]);
    }
  }
  if (tid < D) nm[tid] = n;
  if (tid == 0) nm[D] = m;  // every thread has read the old maximum before the first barrier
}

template <typename T, int VEC>
void launch_walk(const MatrixMemoryParams& p, hipStream_t st) {
  const int CG = p.V / VEC, RG = kWalkThreads / CG, nr = (p.D + RG - 1) / RG;
  const dim3 grid(p.H, p.nseq), block(kWalkThreads);
  const size_t lds = (size_t)(2 * p.D + RG * p.V + 2 * (kWalkThreads / 64)) * sizeof(float);
#define DSSE_WALK(n) hipLaunchKernelGGL((matrix_memory_walk_kernel<T, VEC, n>), grid, block, lds, st, p)
  if (nr <= 2) DSSE_WALK(2);
  else if (nr <= 4) DSSE_WALK(4);
  else if (nr <= 8) DSSE_WALK(8);
  else if (nr <= 16) DSSE_WALK(16);
  else DSSE_WALK(0);
#undef DSSE_WALK
}

// ---------------------------------------------------------------------------------------------------------------------
// Chunk form for prompt portions.  The running maximum only rescales, so it is settled first:
//
//   memory_gates   one wave per (sequence, head), 64 tokens per step: the maximum is a scan of the pairs
//                  (sum of f, best i + later f's); log a_t = f_t + m_(t-1) - m_t and log b_t = i_t - m_t are both <= 0.  Left
//                  behind: A_t = the sum of log a inside its 32-token chunk, u_t = log b_t - A_t, and m_t.
//   memory_chunk   S_t = a_t S_(t-1) + b_t k v^T over chunks of 32 tokens.  For s <= t of one chunk the write of s weighs
//                  e^(A_t + u_s) in t's read-out, the incoming state e^(A_t):
//                      O = e^A (Q S_in) + (Q K^T * W) V,     S_out = e^(A_end) S_in + sum_s e^(A_end + u_s) k_s v_s^T
//   memory_out     division, head norm, gate
//
// memory_chunk: a wave owns 16 columns of one (sequence, head): all D rows of S for them sit in its MFMA accumulators
// (row 4 g + i of tile dt, column r) for the whole portion.  The accumulator layout of S is at the same time the A operand of
// O^T = S^T Q^T (row = column of S, k axis = its rows) when Q's coordinates are staged in the order the accumulators hold
// them, and the accumulator layout of the scores S^T[s, t] is the B operand of O^T += V^T P^T: neither passes through LDS.
// The four waves of a workgroup share the staged q, k (rows, for the scores) and k transposed (for the state's update).
// The normaliser is one more 16-column tile whose "values" are 1 in its first column.
//
// Operands are bf16 where they are projections (q, k, v); what the recurrence makes -- the state, the write strengths, the
// weighted scores -- enters as two bf16 parts (value and remainder), so a product carries about 16 bits of it; sums and the
// state itself are fp32.
constexpr int kChunk = 32;

__global__ __launch_bounds__(64) void memory_gates_kernel(MatrixMemoryParams p) {
  const int h = blockIdx.x, seq = blockIdx.y, lane = threadIdx.x;
  const int ql = p.q_len[seq];
  if (ql <= 0) return;
  const int64_t row0 = p.q_start[seq];
  float* nm = p.norm + ((int64_t)p.state_slot[seq] * p.H + h) * (p.D + 1);
  float m_in = p.ctx_len[seq] - ql == 0 ? 0.0f : nm[p.D];
  const float bi = p.gate_b[h], bf = p.gate_b[p.H + h];
  auto z_at = [&](int t, int c) { return t < ql ? p.gates[(row0 + t) * p.ldz + c * p.H + h] : 0.0f; };
  float zi = z_at(lane, 0), zf = z_at(lane, 1);
  for (int b = 0; b < ql; b += 64) {
    const int t = b + lane;
    const bool on = t < ql;
    const float i = on ? softcap_f(zi + bi, p.cap) : -INFINITY;
    const float f = on ? logsigmoid_f(softcap_f(zf + bf, p.cap)) : 0.0f;
    zi = z_at(t + 64, 0), zf = z_at(t + 64, 1);  // the next step's, in flight over the scans
    float F = f, M = i;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float Fp = __shfl_up(F, o), Mp = __shfl_up(M, o);
      if (lane >= o) {
        M = fmaxf(Mp + F, M);
        F += Fp;
      }
    }
    const float m = fmaxf(m_in + F, M);
    float mp = __shfl_up(m, 1);
    if (lane == 0) mp = m_in;
    float A = on ? f + mp - m : 0.0f;
    const float lb = i - m;
#pragma unroll
    for (int o = 1; o < kChunk; o <<= 1) {
      const float Ap = __shfl_up(A, o);
      if ((lane & (kChunk - 1)) >= o) A += Ap;
    }
    if (on) {
      p.acum[(int64_t)h * p.T + row0 + t] = A;
      p.u[(int64_t)h * p.T + row0 + t] = lb - A;
      p.m[(row0 + t) * p.H + h] = m;
    }
    m_in = __shfl(m, 63);
  }
  if (lane == 0) nm[p.D] = m_in;
}

// value and remainder of fp32 numbers as bf16 operands
DEV void split8(const float (&x)[8], bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    hi[j] = (bf16)x[j];
    lo[j] = (bf16)(x[j] - (float)hi[j]);
  }
}

// NK: 32-row groups of S (D rounded up); NW: waves (16-column tiles) per workgroup
template <int NK, int NW>
__global__ __launch_bounds__(64 * NW) void memory_chunk_kernel(MatrixMemoryParams p) {
  constexpr int Dp = 32 * NK, ldr = Dp + 8, ldt = kChunk + 8;
  constexpr int Q4 = 8 * NK;                  // 4-coordinate pieces of a row
  constexpr int NB = (NK + NW - 1) / NW;      // 4 x 4 pieces (tokens x coordinates) a thread stages
  __shared__ __align__(16) bf16 qs[kChunk * ldr], ks[kChunk * ldr], kt[Dp * ldt];
  const int h = blockIdx.y, seq = blockIdx.z;
  const int ql = p.q_len[seq];
  if (ql <= 0) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int D = p.D, V = p.V;
  const int vtiles = (V + 15) / 16;
  const int ct = blockIdx.x * NW + wave;      // this wave's column tile; vtiles: the normaliser's
  const bool live = ct <= vtiles, is_norm = ct == vtiles;
  const int col = ct * 16 + r;
  const bool col_on = live && !is_norm && col < V;
  const int64_t row0 = p.q_start[seq];
  const bool fresh = p.ctx_len[seq] - ql == 0;
  const int64_t entry = (int64_t)p.state_slot[seq] * p.H + h;
  float* st = p.state + entry * D * V + col;
  float* nm = p.norm + entry * (D + 1);
  f32x4 S[2 * NK];
#pragma unroll
  for (int dt = 0; dt < 2 * NK; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * dt + 4 * g + i;
      float s = 0.0f;
      if (!fresh && d < D) {
        if (col_on) s = st[(int64_t)d * V];
        else if (is_norm && r == 0) s = nm[d];
      }
      S[dt][i] = s;
    }
  // the next chunk's inputs, requested while the current one is in the MFMAs
  f32x4 nk[NB][4], nq[NB][4];
  float nv[8], nu[8], nA0, nA1, nAL;
  const float* Ah = p.acum + (int64_t)h * p.T + row0;
  const float* uh = p.u + (int64_t)h * p.T + row0;
  auto token_of = [&](int j) { return j < 4 ? 4 * g + j : 16 + 4 * g + (j - 4); };  // of k-axis slot (g, j)
  auto ld4 = [&](const float* q) {
    if (p.vec) return ld_global<f32x4>(q);
    return f32x4{q[0], q[1], q[2], q[3]};
  };
  auto request = [&](int t0) {
    const int nt = ql - t0 < kChunk ? ql - t0 : kChunk;
#pragma unroll
    for (int n = 0; n < NB; ++n) {
      const int b = n * 64 * NW + tid, d = 4 * (b % Q4), tq = 4 * (b / Q4);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bool on = tq + j < nt && d < D;
        const int64_t row = row0 + t0 + tq + j;
        nk[n][j] = on ? ld4(p.k + row * p.ldk + h * D + d) : f32x4{0.f, 0.f, 0.f, 0.f};
        nq[n][j] = on ? ld4(p.q + row * p.ldq + h * D + d) : f32x4{0.f, 0.f, 0.f, 0.f};
      }
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int s = token_of(j);
      nv[j] = s >= nt ? 0.0f : (is_norm ? (r == 0 ? 1.0f : 0.0f) : (col_on ? p.v[(row0 + t0 + s) * p.ldv + h * V + col] : 0.0f));
      nu[j] = uh[t0 + (s < nt ? s : nt - 1)];
    }
    nA0 = Ah[t0 + (r < nt ? r : nt - 1)];
    nA1 = Ah[t0 + (16 + r < nt ? 16 + r : nt - 1)];
    nAL = Ah[t0 + nt - 1];
  };
  auto place = [](int x) { return (x & ~31) + ((x & 15) >> 2) * 8 + ((x >> 4) & 1) * 4 + (x & 3); };
  request(0);
  for (int t0 = 0; t0 < ql; t0 += kChunk) {
    const int nt = ql - t0 < kChunk ? ql - t0 : kChunk;
#pragma unroll
    for (int n = 0; n < NB; ++n) {
      const int b = n * 64 * NW + tid;
      if (b < 64 * NK) {
        const int d = 4 * (b % Q4), tq = 4 * (b / Q4);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          bf16x4 qv, kv, kc;
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            qv[e] = (bf16)(nq[n][j][e] * p.q_scale);
            kv[e] = (bf16)nk[n][j][e];
            kc[e] = (bf16)nk[n][e][j];  // coordinate d + j of the four tokens
          }
          *reinterpret_cast<bf16x4*>(qs + (tq + j) * ldr + place(d)) = qv;
          *reinterpret_cast<bf16x4*>(ks + (tq + j) * ldr + place(d)) = kv;
          *reinterpret_cast<bf16x4*>(kt + (d + j) * ldt + place(tq)) = kc;
        }
      }
    }
    float v[8], u[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = nv[j], u[j] = nu[j];
    const float A0 = nA0, A1 = nA1, AL = nAL;
    __syncthreads();
    if (t0 + kChunk < ql) request(t0 + kChunk);
    if (live) {
      f32x4 O0 = f32x4{0.f, 0.f, 0.f, 0.f}, O1 = O0, s00 = O0, s01 = O0, s11 = O0;
#pragma unroll
      for (int k = 0; k < NK; ++k) {
        const bf16x8 q0 = *reinterpret_cast<const bf16x8*>(qs + r * ldr + 32 * k + 8 * g);
        const bf16x8 q1 = *reinterpret_cast<const bf16x8*>(qs + (16 + r) * ldr + 32 * k + 8 * g);
        const bf16x8 k0 = *reinterpret_cast<const bf16x8*>(ks + r * ldr + 32 * k + 8 * g);
        const bf16x8 k1 = *reinterpret_cast<const bf16x8*>(ks + (16 + r) * ldr + 32 * k + 8 * g);
        s00 = mfma16x16x32(k0, q0, s00);
        s01 = mfma16x16x32(k0, q1, s01);
        s11 = mfma16x16x32(k1, q1, s11);
        float x[8];
#pragma unroll
        for (int i = 0; i < 4; ++i) x[i] = S[2 * k][i], x[4 + i] = S[2 * k + 1][i];
        bf16x8 hi, lo;
        split8(x, hi, lo);
        O0 = mfma16x16x32(hi, q0, O0);
        O1 = mfma16x16x32(hi, q1, O1);
        O0 = mfma16x16x32(lo, q0, O0);
        O1 = mfma16x16x32(lo, q1, O1);
      }
      const float e0 = expf(A0), e1 = expf(A1), eL = expf(AL);
      float P0[8], P1[8], vw[8];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        O0[i] *= e0;
        O1[i] *= e1;
        const bool seen = 4 * g + i <= r;
        P0[i] = seen ? s00[i] * expf(A0 + u[i]) : 0.0f;
        P0[4 + i] = 0.0f;
        P1[i] = s01[i] * expf(A1 + u[i]);
        P1[4 + i] = seen ? s11[i] * expf(A1 + u[4 + i]) : 0.0f;
      }
      bf16x8 vb, hi, lo;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        vb[j] = (bf16)v[j];
        vw[j] = v[j] * expf(AL + u[j]);
      }
      split8(P0, hi, lo);
      O0 = mfma16x16x32(vb, hi, O0);
      O0 = mfma16x16x32(vb, lo, O0);
      split8(P1, hi, lo);
      O1 = mfma16x16x32(vb, hi, O1);
      O1 = mfma16x16x32(vb, lo, O1);
      split8(vw, hi, lo);
#pragma unroll
      for (int dt = 0; dt < 2 * NK; ++dt) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(kt + (16 * dt + r) * ldt + 8 * g);
        f32x4 s = S[dt];
#pragma unroll
        for (int i = 0; i < 4; ++i) s[i] *= eL;
        s = mfma16x16x32(kf, hi, s);
        S[dt] = mfma16x16x32(kf, lo, s);
      }
      const int c4 = ct * 16 + 4 * g;  // O^T: rows are columns c4 .. c4 + 3, the lane's token is r (and 16 + r)
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const f32x4 o = b == 0 ? O0 : O1;
        const int t = 16 * b + r;
        if (t >= nt) continue;
        const int64_t at = (row0 + t0 + t) * p.H + h;
        if (is_norm) {
          if (g == 0) p.nq[at] = o[0];
        } else if (V % 4 == 0) {
          if (c4 < V) *reinterpret_cast<f32x4*>(p.num + at * V + c4) = o;
        } else {
#pragma unroll
          for (int i = 0; i < 4; ++i)
            if (c4 + i < V) p.num[at * V + c4 + i] = o[i];
        }
      }
    }
    __syncthreads();  // the staged chunk has been read
  }
#pragma unroll
  for (int dt = 0; dt < 2 * NK; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * dt + 4 * g + i;
      if (d >= D) continue;
      if (col_on) st[(int64_t)d * V] = S[dt][i];
      else if (is_norm && r == 0) nm[d] = S[dt][i];
    }
}

// one wave per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void memory_out_kernel(MatrixMemoryParams p) {
  const int lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (int64_t)p.rows * p.H) return;
  const int64_t row = p.row0 + item / p.H;
  const int h = (int)(item % p.H), V = p.V;
  const int64_t at = row * p.H + h;
  const float* o = p.num + at * V;
  const float inv_den = 1.0f / (fmaxf(fabsf(p.nq[at]), expf(-p.m[at])) + p.den_eps);
  float y[8];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    y[i] = i * 64 + lane < V ? o[i * 64 + lane] * inv_den : 0.0f;
    ss += y[i] * y[i];
  }
  const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)V + p.eps) * p.out_scale;
  const float* gate = p.out_gate + row * p.ldg + h * V;
  T* out = reinterpret_cast<T*>(p.out) + row * p.ldo + h * V;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int c = i * 64 + lane;
    if (c < V) out[c] = (T)(y[i] * inv * p.norm_w[h * V + c] * sigmoid_f(gate[c]));
  }
}

}  // namespace
}  // namespace dsse

extern "C" hipError_t dsse_matrix_memory_walk(const dsse::MatrixMemoryParams* p, hipStream_t st) {
  if (p->nseq <= 0 || p->H <= 0) return hipSuccess;
  if (p->D < 1 || p->V < 1 || p->D > dsse::kWalkThreads || p->V > dsse::kWalkThreads || p->nseq > 65535)
    return hipErrorInvalidValue;
  if (p->V % 4 == 0) {
    if (p->f32) dsse::launch_walk<float, 4>(*p, st);
    else dsse::launch_walk<bf16, 4>(*p, st);
  } else {
    if (p->f32) dsse::launch_walk<float, 1>(*p, st);
    else dsse::launch_walk<bf16, 1>(*p, st);
  }
  return hipGetLastError();
}

extern "C" hipError_t dsse_matrix_memory_chunk(const dsse::MatrixMemoryParams* p, hipStream_t st) {
  if (p->nseq <= 0 || p->H <= 0 || p->rows <= 0) return hipSuccess;
  if (p->f32 || p->D < 1 || p->D > 256 || p->D % 4 || p->V < 1 || p->V > 512 || p->nseq > 65535 || p->H > 65535)
    return hipErrorInvalidValue;
  hipLaunchKernelGGL(dsse::memory_gates_kernel, dim3(p->H, p->nseq), dim3(64), 0, st, *p);
  const int tiles = (p->V + 15) / 16 + 1;
  constexpr int NW = 4;
  const dim3 grid((tiles + NW - 1) / NW, p->H, p->nseq);
  switch ((p->D + 31) / 32) {
#define DSSE_CHUNK_CASE(n) \
  case n: hipLaunchKernelGGL((dsse::memory_chunk_kernel<n, NW>), grid, dim3(64 * NW), 0, st, *p); break;
    DSSE_CHUNK_CASE(1) DSSE_CHUNK_CASE(2) DSSE_CHUNK_CASE(3) DSSE_CHUNK_CASE(4) DSSE_CHUNK_CASE(5) DSSE_CHUNK_CASE(6)
    DSSE_CHUNK_CASE(7) DSSE_CHUNK_CASE(8)
#undef DSSE_CHUNK_CASE
  }
  const long long items = (long long)p->rows * p->H;
  hipLaunchKernelGGL(dsse::memory_out_kernel<bf16>, dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, *p);
  return hipGetLastError();
}
