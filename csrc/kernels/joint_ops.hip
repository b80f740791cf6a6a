// Row-wise pieces of designs whose attention takes the fused projection's q | k | v columns with biases and a per-head
// RMS norm:
//
//   qkv_rows   x + bias; every query and key head divided by its root mean square; queries to a buffer, keys and values
//              into their pages (values once more into the transposed pages) -- one launch instead of one per operand
//
// One wave per (row, head), four heads of a row per workgroup, no barrier: a head of up to 512 coordinates sits in eight
// registers of its wave between the statistic and the write.  Everything is computed in fp32; only page rows of the
// element type are rounded.
#include "api_mixers.h"

namespace dsse {
namespace {

constexpr int kHeadRegs = 8;  // coordinates per lane: heads up to 512 wide

template <typename T>
__global__ __launch_bounds__(256) void qkv_rows_kernel(QkvRowsParams p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int row = blockIdx.x;
  const int head = blockIdx.y * 4 + wave;  // H query heads, then G key heads, then G value heads
  const bool own = p.k != nullptr;
  if (head >= p.H + (own ? 2 * p.G : 0)) return;
  const int part = head < p.H ? 0 : (head < p.H + p.G ? 1 : 2);
  const int h = part == 0 ? head : (part == 1 ? head - p.H : head - p.H - p.G);
  const int D = part == 2 ? p.V : p.D;
  const int col = part == 0 ? h * p.D : (part == 1 ? (p.H + h) * p.D : (p.H + p.G) * p.D + h * p.V);
  int slot = -1;
  if (part != 0) {
    slot = p.slots[row];
    if (slot < 0 || slot >= p.num_slots) return;  // an inactive row: its queries are computed, its pages untouched
  }
  const float* x = p.x + (int64_t)row * p.ldx + col;
  const float* b = p.bias ? p.bias + col : nullptr;
  float v[kHeadRegs];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < kHeadRegs; ++i) {
    const int d = i * 64 + lane;
    v[i] = d < D ? x[d] + (b ? b[d] : 0.0f) : 0.0f;
    ss += v[i] * v[i];
  }
  const float inv = part == 2 ? 1.0f : 1.0f / sqrtf(wave_sum(ss) / (float)D + p.eps);
  if (part == 0) {
    float* q = p.q + ((int64_t)row * p.H + h) * D;
#pragma unroll
    for (int i = 0; i < kHeadRegs; ++i)
      if (i * 64 + lane < D) q[i * 64 + lane] = v[i] * inv;
    return;
  }
  T* dst = (part == 1 ? reinterpret_cast<T*>(p.k) : reinterpret_cast<T*>(p.v)) + ((int64_t)slot * p.G + h) * D;
#pragma unroll
  for (int i = 0; i < kHeadRegs; ++i)
    if (i * 64 + lane < D) dst[i * 64 + lane] = (T)(v[i] * inv);
  if (part == 2 && p.vt) {  // the same numbers where the MFMA attention's value operand wants them
    const int page = slot / kBS, off = slot % kBS;
    const int at = ((off & 15) >> 2) * 8 + ((off >> 4) & 1) * 4 + (off & 3);
    T* vt = reinterpret_cast<T*>(p.vt) + ((int64_t)page * p.G + h) * D * kBS + at;
#pragma unroll
    for (int i = 0; i < kHeadRegs; ++i)
      if (i * 64 + lane < D) vt[(int64_t)(i * 64 + lane) * kBS] = (T)v[i];
  }
}

}  // namespace
}  // namespace dsse

extern "C" hipError_t dsse_qkv_rows(const dsse::QkvRowsParams* p, hipStream_t st) {
  if (p->T <= 0) return hipSuccess;
  if (p->D > 64 * dsse::kHeadRegs || p->V > 64 * dsse::kHeadRegs) return hipErrorInvalidValue;
  const int heads = p->H + (p->k ? 2 * p->G : 0);
  const dim3 grid(p->T, (heads + 3) / 4);
  if (p->f32) hipLaunchKernelGGL(dsse::qkv_rows_kernel<float>, grid, dim3(256), 0, st, *p);
  else hipLaunchKernelGGL(dsse::qkv_rows_kernel<bf16>, grid, dim3(256), 0, st, *p);
  return hipGetLastError();
}
