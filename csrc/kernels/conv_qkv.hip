// A fused q | k | v projection's rows into the attention's operands, for designs whose queries and keys pass a short
// causal convolution over time and / or an interleaved rotation, in one launch:
//
//   y[t, c]  = sum_j taps[c, j] x[t - K + 1 + j, c]        q and k channels; earlier rows come from the slot's tail
//   (a, b)  -> (a cos - b sin, b cos + a sin)              neighbouring coordinates (2i, 2i + 1) of a head, i < half
//   q       *= q_factor[position]
//   k, v    -> their pages (values once more into the transposed pages); without value columns v = y of k, unrotated
//
// A thread owns one coordinate pair of a head (or of a value head) and walks the rows of its work item in blocks of four:
// the block's inputs are requested together, the window of earlier inputs stays in registers, and four tokens of a page
// leave for the transposed value page as one 8-byte store.  Everything is fp32; only page rows are rounded.
#include "api_memory.h"
#include "common.h"

namespace dsse {
namespace {

constexpr int kRowsAhead = 4;

template <typename T>
DEV void st_pair(T* p, float a, float b, bool both) {
  p[0] = (T)a;
  if (both) p[1] = (T)b;
}

DEV int vt_place(int off) { return ((off & 15) >> 2) * 8 + ((off >> 4) & 1) * 4 + (off & 3); }

// KT: taps held in registers (0: no convolution), or -1: any number, inputs read again per row
template <typename T, int KT>
__global__ __launch_bounds__(256) void conv_qkv_rows_kernel(ConvQkvParams p) {
  const int seq = p.work_seq[blockIdx.y];
  const int ql = p.q_len[seq];
  const int t0 = p.work_tile[blockIdx.y] * p.qt;
  if (t0 >= ql) return;
  const int t1 = t0 + p.qt < ql ? t0 + p.qt : ql;
  const int P = (p.D + 1) >> 1, PV = (p.V + 1) >> 1;
  int u = blockIdx.x * blockDim.x + threadIdx.x;
  const int nqk = (p.H + p.G) * P;
  if (u >= nqk + p.G * PV) return;
  const int part = u < p.H * P ? 0 : (u < nqk ? 1 : 2);  // query, key, value coordinates
  const int W = part == 2 ? p.V : p.D, PW = part == 2 ? PV : P;
  u -= part == 2 ? nqk : (part == 1 ? p.H * P : 0);
  const int h = u / PW, i = u - h * PW, d = 2 * i;
  const bool both = d + 1 < W;
  const int C = (p.H + p.G) * p.D;
  const int col = part == 0 ? h * W + d : (part == 1 ? (p.H + h) * W + d : C + h * W + d);
  const int row0 = p.q_start[seq], pos0 = p.ctx_len[seq] - ql;
  const bool fresh = pos0 == 0;  // the sequence starts in this step: nothing before it
  const float* in = p.x + (int64_t)row0 * p.ldx + col;
  const int K = part == 2 ? 0 : (KT >= 0 ? KT : p.K);
  const int Kt = K > 0 ? K - 1 : 0;
  float* tail = Kt > 0 ? p.tail + (int64_t)p.state_slot[seq] * Kt * C + col : nullptr;
  auto input = [&](int t, int c) -> float {  // the projected row t of this step (t >= -Kt), channel col + c
    if (t >= 0) return in[(int64_t)t * p.ldx + c];
    return fresh ? 0.0f : tail[(int64_t)(Kt + t) * C + c];
  };
  constexpr int KR = KT > 0 ? KT : 1;
  float w0[KR], w1[KR], tp0[KR], tp1[KR];  // the last KR inputs and the taps of both channels
  if (KT > 0 && part != 2) {
#pragma unroll
    for (int k = 0; k < KR; ++k) {
      tp0[k] = p.taps[(int64_t)col * KR + k];
      tp1[k] = both ? p.taps[(int64_t)(col + 1) * KR + k] : 0.0f;
    }
#pragma unroll
    for (int k = 1; k < KR; ++k) {
      w0[k] = input(t0 - KR + k, 0);
      w1[k] = both ? input(t0 - KR + k, 1) : 0.0f;
    }
  }
  const bool to_v = part == 2 || (part == 1 && p.V == 0);
  const int VW = p.V == 0 ? p.D : p.V;
  for (int tb = t0; tb < t1; tb += kRowsAhead) {
    const int n = t1 - tb < kRowsAhead ? t1 - tb : kRowsAhead;
    float a[kRowsAhead], b[kRowsAhead], va[kRowsAhead], vb[kRowsAhead];
    int sl[kRowsAhead];
#pragma unroll
    for (int j = 0; j < kRowsAhead; ++j) {
      const int t = tb + (j < n ? j : 0);
      a[j] = in[(int64_t)t * p.ldx];
      b[j] = both ? in[(int64_t)t * p.ldx + 1] : 0.0f;
      sl[j] = part == 0 ? 0 : p.slots[row0 + t];
      if (sl[j] >= p.num_slots) sl[j] = -1;
    }
#pragma unroll
    for (int j = 0; j < kRowsAhead; ++j) {
      if (j >= n) continue;
      const int t = tb + j, pos = pos0 + t;
      float ya = a[j], yb = b[j];
      if (KT > 0 && part != 2) {
#pragma unroll
        for (int k = 0; k + 1 < KR; ++k) w0[k] = w0[k + 1], w1[k] = w1[k + 1];
        w0[KR - 1] = ya, w1[KR - 1] = yb;
        ya = yb = 0.f;
#pragma unroll
        for (int k = 0; k < KR; ++k) ya += tp0[k] * w0[k], yb += tp1[k] * w1[k];
      } else if (KT < 0 && part != 2) {
        ya = yb = 0.f;
        for (int k = 0; k < K; ++k) {
          ya += p.taps[(int64_t)col * K + k] * input(t - Kt + k, 0);
          if (both) yb += p.taps[(int64_t)(col + 1) * K + k] * input(t - Kt + k, 1);
        }
      }
      va[j] = ya, vb[j] = yb;
      if (part == 2) continue;
      if (p.rope && i < p.half) {
        const float2 cs = p.rope[(int64_t)(pos < p.rope_len ? pos : p.rope_len - 1) * p.half + i];
        const float ra = ya * cs.x - yb * cs.y;
        yb = yb * cs.x + ya * cs.y;
        ya = ra;
      }
      if (part == 0) {
        if (p.q_factor) {
          const float f = p.q_factor[pos < p.q_factor_len ? pos : p.q_factor_len - 1];
          ya *= f, yb *= f;
        }
        st_pair(p.q + ((int64_t)(row0 + t) * p.H + h) * p.D + d, ya, yb, both);
      } else if (sl[j] >= 0) {
        st_pair(reinterpret_cast<T*>(p.k) + ((int64_t)sl[j] * p.G + h) * p.D + d, ya, yb, both);
      }
    }
    if (!to_v) continue;
#pragma unroll
    for (int j = 0; j < kRowsAhead; ++j)
      if (j < n && sl[j] >= 0) st_pair(reinterpret_cast<T*>(p.v) + ((int64_t)sl[j] * p.G + h) * VW + d, va[j], vb[j], both);
    if (!p.vt) continue;
    T* vt = reinterpret_cast<T*>(p.vt);
    auto vrow = [&](int slot) { return vt + (((int64_t)(slot / kBS) * p.G + h) * VW + d) * kBS; };
    if (sizeof(T) == 2 && n == kRowsAhead && sl[0] >= 0 && (sl[0] & 3) == 0 && sl[3] == sl[0] + 3) {
      T* dst = vrow(sl[0]) + vt_place(sl[0] % kBS);
      *reinterpret_cast<bf16x4*>(dst) = bf16x4{(bf16)va[0], (bf16)va[1], (bf16)va[2], (bf16)va[3]};
      if (both) *reinterpret_cast<bf16x4*>(dst + kBS) = bf16x4{(bf16)vb[0], (bf16)vb[1], (bf16)vb[2], (bf16)vb[3]};
    } else {
#pragma unroll
      for (int j = 0; j < kRowsAhead; ++j) {
        if (j >= n || sl[j] < 0) continue;
        T* dst = vrow(sl[j]) + vt_place(sl[j] % kBS);
        dst[0] = (T)va[j];
        if (both) dst[kBS] = (T)vb[j];
      }
    }
  }
  if (KT > 1 && p.qt == 1 && part != 2) {  // one row per sequence: the window in registers is the new tail
#pragma unroll
    for (int j = 0; j + 1 < KR; ++j) {
      tail[(int64_t)j * C] = w0[j + 1];
      if (both) tail[(int64_t)j * C + 1] = w1[j + 1];
    }
  } else if (p.qt == 1 && Kt > 0)  // one row per sequence: this thread alone reads and writes its channels of the tail (ascending:
    for (int j = 0; j < Kt; ++j) {  // entry j takes the old entry j + ql, not yet overwritten)
      tail[(int64_t)j * C] = input(ql - Kt + j, 0);
      if (both) tail[(int64_t)j * C + 1] = input(ql - Kt + j, 1);
    }
}

// After every row of the step has read the old tail: the slot's new tail = the step's last K - 1 projected rows.
__global__ __launch_bounds__(256) void conv_qkv_tail_kernel(ConvQkvParams p) {
  const int seq = blockIdx.y;
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  const int ql = p.q_len[seq], C = (p.H + p.G) * p.D, Kt = p.K - 1;
  if (c >= C || ql <= 0) return;
  const bool fresh = p.ctx_len[seq] - ql == 0;
  float* tail = p.tail + (int64_t)p.state_slot[seq] * Kt * C + c;
  const float* in = p.x + (int64_t)p.q_start[seq] * p.ldx + c;
  for (int j = 0; j < Kt; ++j) {
    const int i = ql - Kt + j;
    tail[(int64_t)j * C] = i >= 0 ? in[(int64_t)i * p.ldx] : (fresh ? 0.0f : tail[(int64_t)(Kt + i) * C]);
  }
}

template <typename T>
void launch_conv_qkv(const ConvQkvParams& p, dim3 grid, hipStream_t st) {
#define DSSE_CONV_QKV(k) hipLaunchKernelGGL((conv_qkv_rows_kernel<T, k>), grid, dim3(256), 0, st, p)
  switch (p.K) {
    case 0: DSSE_CONV_QKV(0); break;
    case 1: DSSE_CONV_QKV(1); break;
    case 2: DSSE_CONV_QKV(2); break;
    case 3: DSSE_CONV_QKV(3); break;
    case 4: DSSE_CONV_QKV(4); break;
    default: DSSE_CONV_QKV(-1); break;
  }
#undef DSSE_CONV_QKV
}

}  // namespace
}  // namespace dsse

extern "C" hipError_t dsse_conv_qkv_rows(const dsse::ConvQkvParams* p, hipStream_t st) {
  if (p->nwork <= 0) return hipSuccess;
  if (p->H < 1 || p->G < 1 || p->D < 1 || p->V < 0 || p->K < 0 || p->qt < 1 || (p->K > 1 && !p->tail) || p->nwork > 65535 ||
      p->nseq > 65535)
    return hipErrorInvalidValue;
  const int units = (p->H + p->G) * ((p->D + 1) / 2) + p->G * ((p->V + 1) / 2);
  const dim3 grid((units + 255) / 256, p->nwork);
  if (p->f32) dsse::launch_conv_qkv<float>(*p, grid, st);
  else dsse::launch_conv_qkv<bf16>(*p, grid, st);
  if (p->K > 1 && p->qt > 1)
    hipLaunchKernelGGL(dsse::conv_qkv_tail_kernel, dim3(((p->H + p->G) * p->D + 255) / 256, p->nseq), dim3(256), 0, st, *p);
  return hipGetLastError();
}
