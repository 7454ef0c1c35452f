// Queries, keys and values that pass a short causal convolution each (interface: stack_ops.h): bias, convolution, one RMS
// norm over all query (and all key) rows of the projection, rotation in halves, the K/V store. Everything is float32 up to
// the store. Wave = 64 lanes.
#include <algorithm>

#include "stack_device.h"
#include "stack_ops.h"

namespace omx {
namespace stack {

constexpr int QKV_MAX = 14336;  // columns of q (or k) that a block keeps in LDS

// A block per (row, part): part 0 the queries, 1 the keys, 2 the values. The part's convolution outputs sit in LDS until
// their norm is known. Inputs from before the step's first row of the sequence come from the ring of carried inputs
// (biases already added), which a step of at most CONV_RING_ROWS rows also advances here. TAPS > 0: P.taps is TAPS, a thread
// takes four neighbouring columns with all its loads in flight together (the order of the sums is the same; heads and half the
// rotated dimensions are multiples of four, rows 16-byte aligned); TAPS == 0: anything else, a column per thread.
__device__ __forceinline__ void st4(float* p, f32x4 v) { *(f32x4*)p = v; }
__device__ __forceinline__ void st4(bf16* p, f32x4 v) {
  *(uint2*)p = uint2{f2bf(v[0]) | (uint32_t)f2bf(v[1]) << 16, f2bf(v[2]) | (uint32_t)f2bf(v[3]) << 16};
}
template <typename T, int NT, int TAPS>
__global__ __launch_bounds__(NT) void qkv_conv_kernel(QkvConvParams P, StepRows R) {
  extern __shared__ __attribute__((aligned(16))) float xs[];
  __shared__ float red[NT / 64];
  const int r = blockIdx.x, part = blockIdx.y, tid = threadIdx.x;
  const int nq = P.H * P.D, nk = P.G * P.D, nv = P.G * P.Dv, ch = nq + nk + nv, K = TAPS > 0 ? TAPS : P.taps, half = P.rot_dims / 2;
  const int c0 = part == 0 ? 0 : part == 1 ? nq : nq + nk, n = part == 0 ? nq : part == 1 ? nk : nv;
  const int seq = R.q_seq[r], pos = R.pos[r], slot = R.slot[r];
  int nb = 0;  // rows of the same sequence right before r, up to taps - 1
  while (nb < K - 1 && r - nb - 1 >= 0 && R.q_seq[r - nb - 1] == seq) ++nb;
  float* win = P.ring ? P.window + (long long)seq * P.stride : nullptr;
  float* cs = xs + n;      // [half]
  float* sn = cs + half;
  if (part < 2)
    for (int i = tid; i < half; i += NT) rotary_cs(pos, P.inv_freq[i], P.rot_amp, cs[i], sn[i]);
  const bool keep = win && R.B <= CONV_RING_ROWS;
  float ss = 0.f;
  if constexpr (TAPS > 0) {
    const int reach = min(TAPS - 1, pos);  // nothing precedes position 0
    for (int i = 4 * tid; i < n; i += 4 * NT) {
      const int c = c0 + i;
      const float* x = P.proj + (long long)r * P.ld + c;
      const f32x4 b = P.bias ? *(const f32x4*)(P.bias + c) : f32x4{0.f, 0.f, 0.f, 0.f};
      f32x4 wv[TAPS], in[TAPS];  // the four columns' taps are 4 TAPS neighbouring numbers
#pragma unroll
      for (int j = 0; j < TAPS; ++j) wv[j] = *(const f32x4*)(P.w + (long long)c * TAPS + 4 * j);
#pragma unroll
      for (int back = 0; back < TAPS; ++back) in[back] = *(const f32x4*)(x - (long long)min(back, nb) * P.ld);
      f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int back = TAPS - 1; back >= 0; --back) {
        if (back > reach) continue;
        f32x4 u = in[back] + b;
        if (back > nb) {
          const float* wr = win + (long long)((pos - back) % P.ring) * ch + c;
          u = f32x4{wr[0], wr[1], wr[2], wr[3]};
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          constexpr int last = TAPS - 1;
          acc[e] += wv[(e * TAPS + last - back) / 4][(e * TAPS + last - back) % 4] * u[e];
        }
        if (back == 0 && keep) {
          float* wr = win + (long long)(pos % P.ring) * ch + c;
#pragma unroll
          for (int e = 0; e < 4; ++e) wr[e] = u[e];
        }
      }
      *(f32x4*)(xs + i) = acc;
      ss += acc[0] * acc[0] + acc[1] * acc[1] + acc[2] * acc[2] + acc[3] * acc[3];
    }
  } else {
    for (int i = tid; i < n; i += NT) {
      const int c = c0 + i;
      const float b = P.bias ? P.bias[c] : 0.f;
      const float cur = P.proj[(long long)r * P.ld + c] + b;
      float acc = 0.f;
      for (int back = min(K - 1, pos); back > 0; --back) {  // nothing precedes position 0
        const float in = back <= nb ? P.proj[(long long)(r - back) * P.ld + c] + b : win[(long long)((pos - back) % P.ring) * ch + c];
        acc += P.w[(long long)c * K + K - 1 - back] * in;
      }
      acc += P.w[(long long)c * K + K - 1] * cur;
      if (keep) win[(long long)(pos % P.ring) * ch + c] = cur;
      xs[i] = acc;
      ss += acc * acc;
    }
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const long long blk = slot / R.bs, at = slot % R.bs;
  if (part == 2) {
    if constexpr (TAPS > 0) {
      for (int i = 4 * tid; i < n; i += 4 * NT)
        st4((T*)P.vc + ((blk * P.G + i / P.Dv) * R.bs + at) * P.Dv + i % P.Dv, *(const f32x4*)(xs + i));
      return;
    }
    for (int i = tid; i < n; i += NT) st((T*)P.vc + ((blk * P.G + i / P.Dv) * R.bs + at) * P.Dv + i % P.Dv, xs[i]);
    return;
  }
  float sum = 0.f;
#pragma unroll
  for (int w = 0; w < NT / 64; ++w) sum += red[w];
  const float inv = 1.f / sqrtf(sum / (float)n + P.eps);
  const float* nw = part == 0 ? P.q_norm : P.k_norm;
  if constexpr (TAPS > 0) {
    for (int i = 4 * tid; i < n; i += 4 * NT) {
      const int g = i / P.D, d = i - g * P.D;
      f32x4 v = *(const f32x4*)(xs + i) * inv * *(const f32x4*)(nw + i);
      if (d < 2 * half) {
        const int f = d < half ? d : d - half, j = d < half ? i + half : i - half;  // the pairs' other elements
        const f32x4 o = *(const f32x4*)(xs + j) * inv * *(const f32x4*)(nw + j);
        const f32x4 c = *(const f32x4*)(cs + f), sv = *(const f32x4*)(sn + f);
        v = v * c + (d < half ? -o : o) * sv;
      }
      if (part == 0)
        st4(P.q + (long long)r * P.ld_q + i, v);
      else
        st4((T*)P.kc + ((blk * P.G + g) * R.bs + at) * P.D + d, v);
    }
    return;
  }
  for (int i = tid; i < n; i += NT) {
    const int d = i % P.D;
    float v = xs[i] * inv * nw[i];
    if (d < 2 * half) {
      const int f = d < half ? d : d - half, j = d < half ? i + half : i - half;  // the pair's other element
      const float o = xs[j] * inv * nw[j];
      v = v * cs[f] + (d < half ? -o : o) * sn[f];
    }
    if (part == 0)
      P.q[(long long)r * P.ld_q + i] = v;
    else
      st((T*)P.kc + ((blk * P.G + i / P.D) * R.bs + at) * P.D + d, v);
  }
}
template <typename T, int NT>
static void launch_qkv_conv_nt(const QkvConvParams& P, const StepRows& R, int taps, size_t lds, hipStream_t s) {
  const dim3 grid(R.B, 3);
  if (taps == 4)
    hipLaunchKernelGGL((qkv_conv_kernel<T, NT, 4>), grid, dim3(NT), lds, s, P, R);
  else if (taps == 3)
    hipLaunchKernelGGL((qkv_conv_kernel<T, NT, 3>), grid, dim3(NT), lds, s, P, R);
  else if (taps == 2)
    hipLaunchKernelGGL((qkv_conv_kernel<T, NT, 2>), grid, dim3(NT), lds, s, P, R);
  else
    hipLaunchKernelGGL((qkv_conv_kernel<T, NT, 0>), grid, dim3(NT), lds, s, P, R);
}
template <typename T>
static void launch_qkv_conv(const QkvConvParams& P, const StepRows& R, int taps, size_t lds, hipStream_t s) {
  if (R.B <= 16 && P.H * P.D >= 2048)  // few rows: more threads per row
    launch_qkv_conv_nt<T, 1024>(P, R, taps, lds, s);
  else
    launch_qkv_conv_nt<T, 256>(P, R, taps, lds, s);
}
bool qkv_conv_supported(int H, int G, int D, int Dv) {
  return H > 0 && G > 0 && H % G == 0 && D > 0 && Dv > 0 && (long long)H * D <= QKV_MAX && (long long)G * D <= QKV_MAX &&
         (long long)G * Dv <= QKV_MAX && D <= 1024;
}
void qkv_conv_prepare(const QkvConvParams& P, const StepRows& R, hipStream_t s) {
  const long long ch = (long long)(P.H + P.G) * P.D + (long long)P.G * P.Dv;
  check(R.B > 0 && R.pos && R.slot && R.q_seq && R.bs > 0 && P.proj && P.ld >= ch && P.w && P.q && P.kc && P.vc && P.q_norm && P.k_norm &&
            P.taps >= 1 && (P.taps == 1 || (P.window && P.ring >= P.taps - 1 + CONV_RING_ROWS && P.stride >= P.ring * ch)) &&
            qkv_conv_supported(P.H, P.G, P.D, P.Dv) && P.ld_q >= P.H * P.D && P.rot_dims >= 0 && P.rot_dims % 2 == 0 &&
            P.rot_dims <= P.D && (P.rot_dims == 0 || P.inv_freq),
        "qkv_conv_prepare: bad operands (up to 14336 query, key or value rows)");
  QkvConvParams Q = P;
  if (P.taps == 1) Q.ring = 0;
  const size_t lds = (size_t)(std::max(P.H * P.D, P.G * std::max(P.D, P.Dv)) + P.rot_dims) * sizeof(float);
  const uintptr_t at = (uintptr_t)P.proj | (uintptr_t)P.bias | (uintptr_t)P.w | (uintptr_t)P.q_norm | (uintptr_t)P.k_norm |
                       (uintptr_t)P.q | (uintptr_t)P.kc | (uintptr_t)P.vc;
  const bool vec = P.D % 4 == 0 && P.Dv % 4 == 0 && P.rot_dims % 8 == 0 && P.ld % 4 == 0 && P.ld_q % 4 == 0 && (at & 15) == 0;
  const int taps = vec && P.taps <= 4 ? P.taps : 0;
  if (P.f32)
    launch_qkv_conv<float>(Q, R, taps, lds, s);
  else
    launch_qkv_conv<bf16>(Q, R, taps, lds, s);
  launched("qkv_conv_prepare");
  if (R.B > CONV_RING_ROWS) conv_ring_window(P.proj, P.ld, (int)ch, P.taps, P.bias, P.window, P.stride, P.ring, R, s);
}

}  // namespace stack
}  // namespace omx
