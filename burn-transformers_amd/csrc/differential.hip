// What stands between a differential attention's two maps and its output projection.
// Every head has two rows of attention outputs over the same values, a1 (map 1) and a2 (map 2); the head's row is
//   o = a1 - lambda * a2,   o <- o / sqrt(mean(o^2) + eps) * post
// with the mean over the head's vdim channels, no scale, and one lambda and one `post` for the layer.  The rows come in
// 32-bit (the difference of two nearly equal rows keeps its digits), statistics are 32-bit.
#include "host.h"

struct DifferentialCall {
  int out_dtype;          // element type of `out`: 0 float32, 1 bfloat16
  int tokens;
  int heads;
  int vdim;               // a head's channels
  int pitch;              // columns of one map's row of a head in `in` (at least vdim)
  int out_cols;           // row-major `out`: columns that are written, zeros behind heads * vdim
  int out_rows;           // 0, or `out` is chunk-major with that many rows (activation_offset)
  float lambda;
  float post;
  float eps;
  const float* in;        // [tokens][ld]: map m of head h at columns (2 h + m) * pitch
  int64_t ld;
  void* out;              // [tokens][ld_out]: head h at columns h * vdim
  int64_t ld_out;
};

template <typename T>
__global__ void __launch_bounds__(256) differential_kernel(DifferentialCall c) {
  const int t = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  T* out = static_cast<T*>(c.out);
  for (int head = blockIdx.y * 4 + wave; head < c.heads; head += gridDim.y * 4) {
    const float* first = c.in + (int64_t)t * c.ld + (int64_t)2 * head * c.pitch;
    const float* second = first + c.pitch;
    float squares = 0.f;
    for (int i = lane; i < c.vdim; i += 64) {
      const float v = fmaf(-c.lambda, second[i], first[i]);
      squares = fmaf(v, v, squares);
    }
    const float scale = c.post / sqrtf(wave_sum(squares) / (float)c.vdim + c.eps);
    for (int i = lane; i < c.vdim; i += 64)
      out[activation_offset<T>(c.out_rows, c.ld_out, t, head * c.vdim + i)] = from_float<T>(fmaf(-c.lambda, second[i], first[i]) * scale);
  }
  if (blockIdx.y == 0)
    for (int col = c.heads * c.vdim + threadIdx.x; col < c.out_cols; col += blockDim.x)
      out[activation_offset<T>(c.out_rows, c.ld_out, t, col)] = from_float<T>(0.f);
}

BT_EXPORT int bt_differential_call(void* stream, const DifferentialCall* c) {
  if (c->tokens <= 0) return BT_OK;
  if (c->heads <= 0 || c->vdim <= 0 || c->pitch < c->vdim) BT_REFUSE("differential: %d heads of %d in rows of %d", c->heads, c->vdim, c->pitch);
  const int64_t columns = (int64_t)c->heads * c->vdim;
  if (!c->in || !c->out || c->ld < (int64_t)2 * c->heads * c->pitch || c->out_cols < columns ||
      (c->out_rows == 0 && c->ld_out < c->out_cols) || (c->out_rows != 0 && c->out_rows < c->tokens))
    BT_REFUSE("differential: missing operand or rows too short");
  int per_token = (c->heads + 3) / 4;
  if (per_token > 64) per_token = 64;
  dim3 grid(c->tokens, per_token), block(256);
  if (c->out_dtype == 0)
    hipLaunchKernelGGL(differential_kernel<float>, grid, block, 0, (hipStream_t)stream, *c);
  else
    hipLaunchKernelGGL(differential_kernel<bf16_t>, grid, block, 0, (hipStream_t)stream, *c);
  return bt_check_launch("differential");
}
