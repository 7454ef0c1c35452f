// Gated delta rule (interface: stack_ops.h): per head a float32 state S (D x Dv) whose rows (key channels) decay by a
// per-token vector g, or by one number (head_decay: template parameter HD); a write takes off what the state already
// answers to its key:
//   S <- diag(g_t) S,   u_t = beta_t (v_t - S^T k_t),   S <- S + k_t u_t^T,   o_t = S^T q_t.
// q, k and v come through one short causal convolution with silu; q and k are unit vectors per head (q also times
// D^(-1/2)); g = exp(-exp(A_log) softplus(z)) with z from a low-rank map, the output gate sigmoid of another one; with one
// decay per head z comes straight from the input and the output gate is silu of a full projection.
//   delta_prepare_kernel  convolution, silu, unit vectors, log decays and the output gate of every row (and, for a layer
//                         with an attention beside the delta rule, that attention's K/V store)
//   delta_walk_kernel     token by token, the state in registers (decode steps, and sizes the chunks do not take)
//   delta_wy / scan / out prompt portions in chunks (see there)
// Everything but the matrix operands is float32. Wave = 64 lanes.
#include <hip/hip_runtime.h>
#include <stdint.h>

#include <algorithm>

#include "stack_device.h"
#include "stack_kv.h"
#include "stack_ops.h"

namespace omx {
namespace stack {

constexpr int DELTA_MAX = 256;       // key and value size of a head
constexpr int DELTA_MAX_RANK = 1024;  // both low-rank maps together
__device__ __forceinline__ float delta_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// ------------------------------------------------------------------------------------------------ preparation
// Grid (groups of RB rows, low-rank blocks then convolution blocks). A low-rank block takes 256 outputs (decay
// channels, then gate channels): the rows' first factors sit in LDS, a thread reads its row of the second factor once
// for all RB rows. A convolution block takes four head units (G query heads, G key heads, H value heads), one per
// wave, four channels per lane. Inputs from before the step's first row of the sequence come from its carried window
// (oldest first); a sequence with one row in the step advances its window here, the others in conv_window.
// the input `back` positions before `pos`, from before the step's rows (nb of the sequence's rows precede this one in it)
__device__ __forceinline__ float delta_carried(const DeltaParams& P, const float* win, int back, int nb, int pos, int ch, int c) {
  if (P.ring) return back <= pos ? win[(long long)((pos - back) % P.ring) * ch + c] : 0.f;
  return win[(long long)(P.taps - 1 - (back - nb)) * ch + c];
}
template <typename T, int RB>
__global__ __launch_bounds__(256) void delta_prepare_kernel(DeltaParams P, StepRows R, int nlow) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int r0 = blockIdx.x * RB, nr = min(RB, R.B - r0);
  const int HD = P.H * P.D, HV = P.H * P.Dv, ra = P.rank_a, rg = P.rank_g;
  if ((int)blockIdx.y < nlow) {
    const int ra4 = (ra + 3) / 4 * 4, LR = ra4 + (rg + 3) / 4 * 4;  // both maps' factors 16-byte aligned
    for (int i = tid; i < RB * (ra + rg); i += 256) {
      const int r = i / (ra + rg), c = i % (ra + rg);
      const int col = c < ra ? P.off_a1 + c : P.off_g1 + c - ra;
      lds[r * LR + (c < ra ? c : ra4 + c - ra)] = r < nr ? P.proj[(long long)(r0 + r) * P.ld + col] : 0.f;
    }
    __syncthreads();
    const int c = blockIdx.y * 256 + tid;
    if (c >= HD + HV) return;
    const bool dec = c < HD;
    const int rank = dec ? ra : rg;
    const T* w = dec ? (const T*)P.a2 + (long long)c * ra : (const T*)P.g2 + (long long)(c - HD) * rg;
    const float* x = lds + (dec ? 0 : ra4);
    float z[RB];
#pragma unroll
    for (int r = 0; r < RB; ++r) z[r] = dec ? P.dt_bias[c] : 0.f;
    int i = 0;
    if (sizeof(T) == 2 && rank % 8 == 0 && (((uintptr_t)w) & 15) == 0) {
      for (; i < rank; i += 8) {
        const u32x4 a = *(const u32x4*)(w + i);
        float w8[8];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          w8[2 * u] = __uint_as_float(a[u] << 16);
          w8[2 * u + 1] = __uint_as_float(a[u] & 0xffff0000u);
        }
#pragma unroll
        for (int r = 0; r < RB; ++r) {
          const f32x4 xa = *(const f32x4*)(x + r * LR + i), xb = *(const f32x4*)(x + r * LR + i + 4);
          z[r] += w8[0] * xa[0] + w8[1] * xa[1] + w8[2] * xa[2] + w8[3] * xa[3] + w8[4] * xb[0] + w8[5] * xb[1] + w8[6] * xb[2] +
                  w8[7] * xb[3];
        }
      }
    }
    for (; i < rank; ++i) {
      const float w0 = ld(w + i);
#pragma unroll
      for (int r = 0; r < RB; ++r) z[r] += w0 * x[r * LR + i];
    }
    const float ea = dec ? expf(P.a_log[c / P.D]) : 0.f;
#pragma unroll
    for (int r = 0; r < RB; ++r)
      if (r < nr) {
        if (dec)
          P.lg[(long long)(r0 + r) * P.ld_lg + c] = -ea * delta_softplus(z[r]);
        else
          P.gate[(long long)(r0 + r) * P.ld_gate + c - HD] = sigmoidf(z[r]);
      }
    return;
  }
  const int unit = ((int)blockIdx.y - nlow) * 4 + wv;
  if (unit >= 2 * P.G + P.H) {  // past the head units: the attention's K/V store, a wave per key/value head
    const int g = unit - 2 * P.G - P.H;
    if (P.kv.kc && g < P.kv.G)
      for (int rr = 0; rr < nr; ++rr) kv_store_item<T>(P.kv, R, r0 + rr, g, lane);
    return;
  }
  const bool isv = unit >= 2 * P.G, isq = unit < P.G;
  if (P.head_decay && isv && lane < nr) {  // the head's log decays, a row per lane
    const int h = unit - 2 * P.G;
    const long long r = r0 + lane;
    P.lg[r * P.ld_lg + h] = -expf(P.a_log[h]) * delta_softplus(P.proj[r * P.ld + P.off_a1 + h] + P.dt_bias[h]);
  }
  const int n = isv ? P.Dv : P.D, K = P.taps;
  const int c0 = isv ? 2 * P.G * P.D + (unit - 2 * P.G) * P.Dv : unit * P.D;  // first channel of the unit
  const int ch = 2 * P.G * P.D + HV;
  if (RB > 1 && K <= 4) {  // prompt portions: a channel's inputs of all rows (and the three before) requested at once
    float v[DELTA_MAX / 64][RB];
#pragma unroll
    for (int u = 0; u < DELTA_MAX / 64; ++u) {
      const int d = lane + 64 * u;
      if (64 * u < n) {  // uniform over the wave
        const int c = c0 + min(d, n - 1);
        float in[RB + 3], w[4];
#pragma unroll
        for (int i = 0; i < RB + 3; ++i) in[i] = P.proj[(long long)min(max(r0 - 3 + i, 0), R.B - 1) * P.ld + P.off_q + c];
#pragma unroll
        for (int b = 0; b < 4; ++b) w[b] = b < K ? P.conv_w[(long long)c * K + (K - 1 - b)] : 0.f;  // w[back]
#pragma unroll
        for (int rr = 0; rr < RB; ++rr) {
          const int r = min(r0 + rr, R.B - 1), seq = R.q_seq[r];
          int nb = 0;
          while (nb < K - 1 && r - nb - 1 >= 0 && R.q_seq[r - nb - 1] == seq) ++nb;
          const bool alone = nb == 0 && !(r + 1 < R.B && R.q_seq[r + 1] == seq);
          float* win = P.window + (long long)seq * P.state_stride;
          float acc = 0.f;
#pragma unroll
          for (int back = 3; back >= 0; --back)
            if (back < K) acc += w[back] * (back <= nb ? in[rr + 3 - back] : delta_carried(P, win, back, nb, R.pos[r], ch, c));
          if (alone && rr < nr && d < n && !P.ring)  // (rings: conv_ring_window)
            for (int sx = 0; sx < K - 1; ++sx)
              win[(long long)sx * ch + c] = sx == K - 2 ? in[rr + 3] : win[(long long)(sx + 1) * ch + c];
          v[u][rr] = d < n ? silu(acc) : 0.f;
        }
      } else {
#pragma unroll
        for (int rr = 0; rr < RB; ++rr) v[u][rr] = 0.f;
      }
    }
#pragma unroll
    for (int rr = 0; rr < RB; ++rr) {
      if (rr >= nr) break;  // uniform over the block
      float f = 1.f;
      if (!isv) {
        float ss = 0.f;
#pragma unroll
        for (int u = 0; u < DELTA_MAX / 64; ++u) ss += v[u][rr] * v[u][rr];
        f = (isq ? 1.f / sqrtf((float)P.D) : 1.f) / sqrtf(wave_sum(ss) + 1e-6f);
      }
#pragma unroll
      for (int u = 0; u < DELTA_MAX / 64; ++u) {
        const int d = lane + 64 * u;
        if (d < n) P.x[(long long)(r0 + rr) * P.ld_x + c0 + d] = v[u][rr] * f;
      }
    }
    return;
  }
  for (int rr = 0; rr < nr; ++rr) {
    const int r = r0 + rr, seq = R.q_seq[r];
    int nb = 0;  // rows of the same sequence right before r, up to taps - 1
    while (nb < K - 1 && r - nb - 1 >= 0 && R.q_seq[r - nb - 1] == seq) ++nb;
    const bool alone = nb == 0 && !(r + 1 < R.B && R.q_seq[r + 1] == seq);
    float* win = P.window + (long long)seq * P.state_stride;
    float v[DELTA_MAX / 64], ss = 0.f;
#pragma unroll
    for (int u = 0; u < DELTA_MAX / 64; ++u) {
      const int d = lane + 64 * u;
      v[u] = 0.f;
      if (d < n) {
        const int c = c0 + d;
        const float cur = P.proj[(long long)r * P.ld + P.off_q + c];
        float acc = 0.f;
        for (int j = 0; j < K; ++j) {
          const int back = K - 1 - j;
          const float in = back == 0 ? cur : back <= nb ? P.proj[(long long)(r - back) * P.ld + P.off_q + c]
                                                        : delta_carried(P, win, back, nb, R.pos[r], ch, c);
          acc += P.conv_w[(long long)c * K + j] * in;
          if (P.ring) {
            if (back == 0 && R.B <= CONV_RING_ROWS) win[(long long)(R.pos[r] % P.ring) * ch + c] = cur;
          } else if (alone && back > 0) win[(long long)(K - 1 - back) * ch + c] = back == 1 ? cur : win[(long long)(K - back) * ch + c];
        }
        v[u] = silu(acc);
        ss += v[u] * v[u];
      }
    }
    float f = 1.f;
    if (!isv) f = (isq ? 1.f / sqrtf((float)P.D) : 1.f) / sqrtf(wave_sum(ss) + 1e-6f);
#pragma unroll
    for (int u = 0; u < DELTA_MAX / 64; ++u) {
      const int d = lane + 64 * u;
      if (d < n) P.x[(long long)r * P.ld_x + c0 + d] = v[u] * f;
    }
  }
}
template <typename T>
static void launch_delta_prepare(const DeltaParams& P, const StepRows& R, hipStream_t s) {
  const int nlow = P.head_decay ? 0 : (P.H * (P.D + P.Dv) + 255) / 256, nconv = (2 * P.G + P.H + (P.kv.kc ? P.kv.G : 0) + 3) / 4;
  const int rank = P.head_decay ? 0 : (P.rank_a + 3) / 4 * 4 + (P.rank_g + 3) / 4 * 4;
  if (R.B <= 16)
    hipLaunchKernelGGL((delta_prepare_kernel<T, 1>), dim3(R.B, nlow + nconv), dim3(256), rank * 4, s, P, R, nlow);
  else
    hipLaunchKernelGGL((delta_prepare_kernel<T, 8>), dim3((R.B + 7) / 8, nlow + nconv), dim3(256), 8 * rank * 4, s, P, R, nlow);
}
bool delta_supported(int D, int Dv, int rank_a, int rank_g) {
  return D > 0 && Dv > 0 && D <= DELTA_MAX && Dv <= DELTA_MAX && rank_a > 0 && rank_g > 0 && rank_a + rank_g <= DELTA_MAX_RANK;
}
bool delta_head_supported(int D, int Dv) { return D > 0 && Dv > 0 && D <= DELTA_MAX && Dv <= DELTA_MAX; }
static void check_delta(const DeltaParams& P, const StepRows& R) {
  const bool maps = P.head_decay ? delta_head_supported(P.D, P.Dv)
                                 : P.a2 && P.g2 && P.gate && P.ld_lg >= P.H * P.D && delta_supported(P.D, P.Dv, P.rank_a, P.rank_g);
  check(R.B > 0 && P.proj && P.conv_w && P.a_log && P.dt_bias && P.norm_w && P.state && P.out && P.x && P.lg && P.G > 0 &&
            P.H % P.G == 0 && P.taps >= 1 && (P.taps == 1 || P.window) && maps && P.ld_x >= 2 * P.G * P.D + P.H * P.Dv &&
            P.ld_lg >= P.H && P.ld_gate >= P.H * P.Dv && P.ld_out >= P.H * P.Dv &&
            (P.ring == 0 || P.taps == 1 || (R.pos && P.ring >= P.taps - 1 + CONV_RING_ROWS)),
        "gated delta rule: operands or head sizes (key and value size <= 256)");
}
void delta_prepare(const DeltaParams& P, const StepRows& R, hipStream_t s) {
  check_delta(P, R);
  check(!P.kv.kc || (P.kv.proj && P.kv.vc && P.kv.G > 0 && P.kv.D > 0 && P.kv.Dv > 0 && P.kv.f32 == P.f32 && R.slot && R.bs > 0),
        "delta_prepare: K/V store operands");
  if (P.f32)
    launch_delta_prepare<float>(P, R, s);
  else
    launch_delta_prepare<bf16>(P, R, s);
  launched("delta_prepare");
  const int ch = 2 * P.G * P.D + P.H * P.Dv;
  if (P.ring) {
    if (R.B > CONV_RING_ROWS) conv_ring_window(P.proj + P.off_q, P.ld, ch, P.taps, nullptr, P.window, P.state_stride, P.ring, R, s);
    return;
  }
  ConvParams C{P.proj, P.ld, P.off_q, ch, P.taps, P.conv_w, nullptr, P.window, P.state_stride, nullptr, 0};
  conv_window(C, R, s);
}

template <bool HD>
__device__ __forceinline__ float delta_gate(const DeltaParams& P, long long r, int i) {  // output gate of value channel i
  return HD ? silu(P.proj[r * P.ld + P.off_g1 + i]) : P.gate[r * P.ld_gate + i];
}
// ------------------------------------------------------------------------------------------------ token by token
// One block per (sequence segment of the step, head), as the other recurrences: the block of the segment's first row
// walks its rows; thread (g, j) = (tid / Dv, tid % Dv) keeps S[i][j], i = g, g + NG, ..., in registers. The head's RMS
// norm, its weight and the gate finish the row.
template <typename T, int MAXI, int NT, bool HD>
__global__ __launch_bounds__(NT) void delta_walk_kernel(DeltaParams P, StepRows R) {
  __shared__ float qs[DELTA_MAX], ks[DELTA_MAX], gs[DELTA_MAX], us[DELTA_MAX], po[NT], red[4];
  const int r0 = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int seq = R.q_seq[r0];
  if (r0 > 0 && R.q_seq[r0 - 1] == seq) return;  // not the first row of its segment (uniform per block)
  const int D = P.D, Dv = P.Dv, hg = h / (P.H / P.G);
  const int NG = NT / Dv;
  const int g = tid / Dv, j = tid % Dv;
  const bool act = g < NG;
  float* S0 = P.state + (long long)seq * P.state_stride + (long long)h * D * Dv;
  float S[MAXI];
#pragma unroll
  for (int ii = 0; ii < MAXI; ++ii) {
    const int i = g + ii * NG;
    S[ii] = (act && i < D) ? S0[(long long)i * Dv + j] : 0.f;
  }
  for (int r = r0; r < R.B && R.q_seq[r] == seq; ++r) {
    const float* x = P.x + (long long)r * P.ld_x;
    if (tid < D) {
      qs[tid] = x[hg * D + tid];
      ks[tid] = x[P.G * D + hg * D + tid];
      gs[tid] = expf(P.lg[(long long)r * P.ld_lg + (HD ? h : h * D + tid)]);
    }
    const float v = tid < Dv ? x[2 * P.G * D + h * Dv + tid] : 0.f;
    const float beta = sigmoidf(P.proj[(long long)r * P.ld + P.off_b + h]);
    const float gate = tid < Dv ? delta_gate<HD>(P, r, h * Dv + tid) : 0.f;
    __syncthreads();
    float part = 0.f;
    if (act) {
#pragma unroll
      for (int ii = 0; ii < MAXI; ++ii) {
        const int i = g + ii * NG;
        if (i < D) {
          S[ii] *= gs[i];
          part += S[ii] * ks[i];
        }
      }
    }
    po[tid] = part;
    __syncthreads();
    if (tid < Dv) {
      float a = 0.f;
      for (int gg = 0; gg < NG; ++gg) a += po[gg * Dv + tid];
      us[tid] = beta * (v - a);
    }
    __syncthreads();
    part = 0.f;
    if (act) {
      const float u = us[j];
#pragma unroll
      for (int ii = 0; ii < MAXI; ++ii) {
        const int i = g + ii * NG;
        if (i < D) {
          S[ii] += ks[i] * u;
          part += S[ii] * qs[i];
        }
      }
    }
    po[tid] = part;
    __syncthreads();
    float o = 0.f;
    if (tid < Dv)
      for (int gg = 0; gg < NG; ++gg) o += po[gg * Dv + tid];
    if (tid < 256) {
      const float w = wave_sum(o * o);
      if ((tid & 63) == 0) red[tid >> 6] = w;
    }
    __syncthreads();
    if (tid < Dv) {
      const float ms = (red[0] + red[1] + red[2] + red[3]) / (float)Dv;
      st((T*)P.out + (long long)r * P.ld_out + h * Dv + tid, o / sqrtf(ms + P.eps) * P.norm_w[tid] * gate * P.out_scale);
    }
    __syncthreads();
  }
#pragma unroll
  for (int ii = 0; ii < MAXI; ++ii) {
    const int i = g + ii * NG;
    if (act && i < D) S0[(long long)i * Dv + j] = S[ii];
  }
}
template <typename T, bool HD>
static void launch_delta_walk(const DeltaParams& P, const StepRows& R, hipStream_t s) {
  const dim3 grid(R.B, P.H);
  const int ng = 1024 / P.Dv, ni = (P.D + ng - 1) / ng;
  if (P.D * P.Dv <= 2048 && (P.D + 256 / P.Dv - 1) / (256 / P.Dv) <= 8)
    hipLaunchKernelGGL((delta_walk_kernel<T, 8, 256, HD>), grid, dim3(256), 0, s, P, R);
  else if (ni <= 4)
    hipLaunchKernelGGL((delta_walk_kernel<T, 4, 1024, HD>), grid, dim3(1024), 0, s, P, R);
  else if (ni <= 8)
    hipLaunchKernelGGL((delta_walk_kernel<T, 8, 1024, HD>), grid, dim3(1024), 0, s, P, R);
  else if (ni <= 16)
    hipLaunchKernelGGL((delta_walk_kernel<T, 16, 1024, HD>), grid, dim3(1024), 0, s, P, R);
  else if (ni <= 32)
    hipLaunchKernelGGL((delta_walk_kernel<T, 32, 1024, HD>), grid, dim3(1024), 0, s, P, R);
  else
    hipLaunchKernelGGL((delta_walk_kernel<T, 64, 1024, HD>), grid, dim3(1024), 0, s, P, R);
}
void delta_walk(const DeltaParams& P, const StepRows& R, hipStream_t s) {
  check_delta(P, R);
  if (P.f32 && P.head_decay)
    launch_delta_walk<float, true>(P, R, s);
  else if (P.f32)
    launch_delta_walk<float, false>(P, R, s);
  else if (P.head_decay)
    launch_delta_walk<bf16, true>(P, R, s);
  else
    launch_delta_walk<bf16, false>(P, R, s);
  launched("delta_walk");
}

// ------------------------------------------------------------------------------------------------ prompt portions
// Chunks of DC tokens over the host-built chunk table {first row, rows, state slot, flags}. With l_s = ln g_s (a
// vector over the key channels), L_t = l_0 + ... + l_t inside a chunk of n tokens that starts from state S,
//   A[t][s] = beta_t sum_d k_t[d] k_s[d] exp(L_t[d] - L_s[d])  (s < t),   B[t][s] = the same with q_t, no beta (s <= t),
//   u_t = beta_t v_t - beta_t S^T (k_t exp(L_t)) - sum_(s < t) A[t][s] u_s,
// so (I + A) u = beta v - (beta k exp(L)) S: one forward substitution over the columns of both right-hand sides gives
// u = V' - W S with V', W free of the state. Then
//   o_t = S^T (q_t exp(L_t)) + sum_(s <= t) B[t][s] u_s,      S <- diag(exp(L_(n-1))) S + sum_s (k_s exp(L_(n-1) - L_s)) u_s^T.
// Every exponent is <= 0. Float32 throughout; the products over the state on v_mfma_f32_16x16x4_f32 (true float32).
//   delta_wy_kernel    (chunk, head): L (over the log decays), A, B, V' (into u), W, the keys decayed to the chunk's end
//   delta_scan_kernel  (sequence, head, 16 value columns): walks the chunks, u = V' - W S, every chunk's incoming state
//   delta_out_kernel   (chunk, head): the outputs, their norm and gate
constexpr int DC = 32;
constexpr int DELTA_CD = 128;  // largest key size of the chunked form
int delta_chunk_rows() { return DC; }
bool delta_chunk_supported(int D, int Dv) { return D > 0 && D <= DELTA_CD && Dv > 0 && Dv <= DELTA_MAX; }
constexpr int DELTA_WY_MAX = DELTA_CD + DELTA_MAX;
static inline size_t delta_wy_lds(int D, int Dv) {
  return (size_t)(std::max(3 * DC * (D + 1), DC * (D + Dv)) + DC * (DC + 4) + DC) * sizeof(float);
}

template <bool HD>
__global__ __launch_bounds__(DELTA_WY_MAX) void delta_wy_kernel(DeltaParams P, DeltaChunkWs W) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int r0 = W.chunks[4 * c], n = W.chunks[4 * c + 1];
  const int D = P.D, Dv = P.Dv, D1 = D + 1, hg = h / (P.H / P.G);
  const int nt = blockDim.x;         // at least D + Dv: a thread per column of the right-hand sides
  constexpr int LA = DC + 4;       // rows of A 16-byte aligned
  float* A = lds;                  // [DC][DC + 4]
  float* be = A + DC * LA;         // [DC]
  float* qs = be + DC;             // [DC][D + 1]
  float* ks = qs + DC * D1;
  float* Lc = ks + DC * D1;        // [DC][D + 1], or [DC] with one decay per head
  for (int i = tid; i < DC * D; i += nt) {
    const int t = i / D, d = i % D;
    const long long r = r0 + min(t, n - 1);  // (unconditional loads: all of them in flight together)
    const float qv = P.x[r * P.ld_x + hg * D + d], kv = P.x[r * P.ld_x + (P.G + hg) * D + d];
    qs[t * D1 + d] = t < n ? qv : 0.f;
    ks[t * D1 + d] = t < n ? kv : 0.f;
    if constexpr (!HD) {
      const float lv = P.lg[r * P.ld_lg + h * D + d];
      Lc[t * D1 + d] = t < n ? lv : 0.f;
    }
  }
  if (HD && tid < 64) {  // the running log decays: one lane per token
    float v = tid < n ? P.lg[(long long)(r0 + tid) * P.ld_lg + h] : 0.f;
#pragma unroll
    for (int o = 1; o < DC; o <<= 1) {
      const float u = __shfl_up(v, o, 64);
      if (tid >= o) v += u;
    }
    if (tid < DC) Lc[tid] = v;
    if (tid < n) P.lg[(long long)(r0 + tid) * P.ld_lg + h] = v;
  }
  if (tid < DC) be[tid] = tid < n ? sigmoidf(P.proj[(long long)(r0 + tid) * P.ld + P.off_b + h]) : 0.f;
  __syncthreads();
  if constexpr (HD) {
    // A and B are plain products with a factor per pair: a 16 x 16 tile of both per wave (the tile above the diagonal is 0)
    if (tid < 256) {
      const int lane = tid & 63, m = lane & 15, q4 = lane >> 4, mt = tid >> 7, nt2 = (tid >> 6) & 1;
      f32x4 aa = f32x4{0.f, 0.f, 0.f, 0.f}, bb = aa;
      if (nt2 <= mt) {
        const float *kr = ks + (16 * mt + m) * D1, *qr = qs + (16 * mt + m) * D1, *kc = ks + (16 * nt2 + m) * D1;
        for (int d0 = 0; d0 < D; d0 += 4) {
          const int d = min(d0 + q4, D - 1);
          const float kb = d0 + q4 < D ? kc[d] : 0.f;
          aa = __builtin_amdgcn_mfma_f32_16x16x4f32(kr[d], kb, aa, 0, 0, 0);
          bb = __builtin_amdgcn_mfma_f32_16x16x4f32(qr[d], kb, bb, 0, 0, 0);
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 16 * mt + 4 * q4 + i, sx = 16 * nt2 + m;
        const float e = (sx <= t && t < n) ? __builtin_amdgcn_exp2f((Lc[t] - Lc[sx]) * 1.44269504088896341f) : 0.f;
        A[t * LA + sx] = sx < t ? be[t] * aa[i] * e : 0.f;
        if (t < n) W.Bm[((long long)(r0 + t) * P.H + h) * DC + sx] = bb[i] * e;
      }
    }
  } else {
    if (tid < D) {
      float acc = 0.f;
#pragma unroll 8
      for (int t = 0; t < DC; ++t) {
        acc += Lc[t * D1 + tid];
        Lc[t * D1 + tid] = acc;
      }
    }
    __syncthreads();
    for (int i = tid; i < n * D; i += nt) {  // the running log decays replace the log decays
      const int t = i / D, d = i % D;
      P.lg[(long long)(r0 + t) * P.ld_lg + h * D + d] = Lc[t * D1 + d];
    }
    for (int p = tid; p < DC * DC; p += nt) {
      const int t = p / DC, sx = p % DC;
      float a = 0.f, b = 0.f;
      if (sx <= t && t < n) {
        for (int d = 0; d < D; ++d) {  // exponents <= 0; exp2 on the transcendental unit (1 ulp)
          const float e = ks[sx * D1 + d] * __builtin_amdgcn_exp2f((Lc[t * D1 + d] - Lc[sx * D1 + d]) * 1.44269504088896341f);
          a += ks[t * D1 + d] * e;
          b += qs[t * D1 + d] * e;
        }
      }
      A[t * LA + sx] = sx < t ? be[t] * a : 0.f;
      if (t < n) W.Bm[((long long)(r0 + t) * P.H + h) * DC + sx] = b;
    }
  }
  for (int i = tid; i < n * D; i += nt) {  // keys decayed to the end of the chunk
    const int t = i / D, d = i % D;
    const float e = HD ? Lc[n - 1] - Lc[t] : Lc[(n - 1) * D1 + d] - Lc[t * D1 + d];
    W.Kd[(long long)(r0 + t) * W.ld_w + h * D + d] = ks[t * D1 + d] * expf(e);
  }
  __syncthreads();
  // forward substitution, a column of the right-hand sides per thread, in blocks of eight rows: the solved rows sit in LDS
  // (where q, k and the log decays were), so a thread holds sixteen values at a time
  const int col = tid, NC = D + Dv;
  const bool key = col < D;
  float x[DC];
  if (key) {
#pragma unroll
    for (int t = 0; t < DC; ++t)
      x[t] = be[t] * ks[t * D1 + col] * __builtin_amdgcn_exp2f((HD ? Lc[t] : Lc[t * D1 + col]) * 1.44269504088896341f);
  } else if (col < NC) {
    const unsigned at = 2 * P.G * D + h * Dv + col - D;
#pragma unroll
    for (int t = 0; t < DC; ++t) {
      const float* row = P.x + (long long)(r0 + min(t, n - 1)) * P.ld_x;  // (uniform)
      x[t] = row[at];
    }
#pragma unroll
    for (int t = 0; t < DC; ++t) x[t] *= be[t];  // 0 past the chunk's end
  }
  __syncthreads();
  if (col >= NC) return;
  float* X = qs + col;  // [DC][D + Dv]
#pragma unroll
  for (int t = 0; t < DC; ++t) X[t * NC] = x[t];
  float* out = key ? W.W + (long long)r0 * W.ld_w + h * D + col : W.u + (long long)r0 * P.ld_gate + h * Dv + col - D;
  const int ldo = key ? W.ld_w : P.ld_gate;
#pragma unroll 1
  for (int b0 = 0; b0 < n; b0 += 8) {
    float y[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) y[i] = X[(b0 + i) * NC];
#pragma unroll 1
    for (int s0 = 0; s0 < b0; s0 += 8) {
      float z[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) z[i] = X[(s0 + i) * NC];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const f32x4 a = *(const f32x4*)&A[(b0 + i) * LA + s0], c4 = *(const f32x4*)&A[(b0 + i) * LA + s0 + 4];
        y[i] -= a[0] * z[0] + a[1] * z[1] + a[2] * z[2] + a[3] * z[3] + c4[0] * z[4] + c4[1] * z[5] + c4[2] * z[6] + c4[3] * z[7];
      }
    }
#pragma unroll
    for (int i = 1; i < 8; ++i) {
#pragma unroll
      for (int k = 0; k < 7; ++k)
        if (k < i) y[i] -= A[(b0 + i) * LA + b0 + k] * y[k];
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      X[(b0 + i) * NC] = y[i];
      if (b0 + i < n) *out = y[i];
      out += ldo;
    }
  }
}

// Four waves share the state's rows: wave w holds the 16-row tiles w and w + 4 of S (16 columns) in accumulator layout,
// S[16 tile + 4 (lane / 16) + i][lane % 16]. In that layout a register is a B operand of the first product if its K
// order is d = 4 (lane / 16) + i, so W's rows are read four consecutive channels per lane and the state never moves.
// The next chunk's operands are requested before the current chunk is multiplied, always (the last chunk asks for its own
// again: a fetch under a condition would make every later wait a wait for all of it), in two register sets that take turns.
// Indexes past the chunk or the head are clamped: a row past the chunk's end meets u = 0, a channel past the head a key of 0.
template <int TJ>
struct DeltaOps {
  float wa[TJ][2][4], kd[TJ][8], el[TJ][4], vp[2];
};
template <int TJ, bool VEC, bool HD>
__device__ __forceinline__ void delta_fetch(const DeltaParams& P, const DeltaChunkWs& W, int r0, int n, int h, int ct,
                                            DeltaOps<TJ>& o) {
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, m = lane & 15, q4 = lane >> 4, D = P.D;
#pragma unroll
  for (int j = 0; j < TJ; ++j) {
    const int dt = 16 * (wv + 4 * j), dq = dt + 4 * q4;
#pragma unroll
    for (int mt = 0; mt < 2; ++mt) {
      const float* wr = W.W + (long long)(r0 + min(16 * mt + m, n - 1)) * W.ld_w + h * D;
      if constexpr (VEC) {
        const f32x4 a = *(const f32x4*)(wr + min(dq, D - 4));
#pragma unroll
        for (int i = 0; i < 4; ++i) o.wa[j][mt][i] = a[i];
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) o.wa[j][mt][i] = wr[min(dq + i, D - 1)];
      }
    }
#pragma unroll
    for (int kk = 0; kk < 8; ++kk)
      o.kd[j][kk] = W.Kd[(long long)(r0 + min(4 * kk + q4, n - 1)) * W.ld_w + h * D + min(dt + m, D - 1)];
    const float* lr = P.lg + (long long)(r0 + n - 1) * P.ld_lg + (HD ? h : h * D);
#pragma unroll
    for (int i = 0; i < 4; ++i) o.el[j][i] = lr[HD ? 0 : min(dq + i, D - 1)];
  }
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    const int e = tid + 256 * k;
    o.vp[k] = W.u[(long long)(r0 + min(e >> 4, n - 1)) * P.ld_gate + h * P.Dv + min(ct * 16 + (e & 15), P.Dv - 1)];
  }
}
template <int TJ, bool VEC, bool HD>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaParams P, DeltaChunkWs W) {
  __shared__ float part[4][DC][17];
  __shared__ float us[DC][17];
  // grid (head + heads * column tile, chunk): the working blocks (first chunks) are neighbours and so spread over the XCDs, a
  // head's column tiles, which read the same W and keys, stay on one of them (8 | heads)
  const int c0 = blockIdx.y, h = blockIdx.x % P.H, ct = blockIdx.x / P.H, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  if (!(W.chunks[4 * c0 + 3] & 1)) return;  // not the first chunk of its sequence (uniform per block)
  const int D = P.D, Dv = P.Dv, m = lane & 15, q4 = lane >> 4;
  const int col = ct * 16 + m;
  const bool cok = col < Dv;
  float* S0 = P.state + (long long)W.chunks[4 * c0 + 2] * P.state_stride + (long long)h * D * Dv;
  f32x4 S[TJ];
#pragma unroll
  for (int j = 0; j < TJ; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * (wv + 4 * j) + 4 * q4 + i;
      const float v = S0[(long long)min(d, D - 1) * Dv + min(col, Dv - 1)];
      S[j][i] = (cok && d < D) ? v : 0.f;
    }
  int c = c0, r0 = W.chunks[4 * c0], n = W.chunks[4 * c0 + 1], flags = W.chunks[4 * c0 + 3];
  int cn = min(c0 + 1, W.nchunks - 1), r0n = W.chunks[4 * cn], nn = W.chunks[4 * cn + 1], fn = W.chunks[4 * cn + 3];
  DeltaOps<TJ> opa, opb;
  delta_fetch<TJ, VEC, HD>(P, W, r0, n, h, ct, opa);
  auto step = [&](DeltaOps<TJ>& cur, DeltaOps<TJ>& nxt) {
    const bool last = (flags & 2) != 0;  // the sequence's last chunk of the step
    delta_fetch<TJ, VEC, HD>(P, W, last ? r0 : r0n, last ? n : nn, h, ct, nxt);
    cn = min(c + 2, W.nchunks - 1);      // the table's entry after the next one
    const int r0m = W.chunks[4 * cn], nm = W.chunks[4 * cn + 1], fm = W.chunks[4 * cn + 3];
    float* Sin = W.Sin + (long long)c * W.s_stride + (long long)h * D * Dv;
#pragma unroll
    for (int j = 0; j < TJ; ++j)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * (wv + 4 * j) + 4 * q4 + i;
        if (cok && d < D) Sin[(long long)d * Dv + col] = S[j][i];
      }
#pragma unroll
    for (int mt = 0; mt < 2; ++mt) {
      f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < TJ; ++j)
#pragma unroll
        for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.wa[j][mt][i], S[j][i], acc, 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) part[wv][16 * mt + 4 * q4 + i][m] = acc[i];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      const int e = tid + 256 * k, t = e >> 4, cm = e & 15;
      const float u = cur.vp[k] - (part[0][t][cm] + part[1][t][cm] + part[2][t][cm] + part[3][t][cm]);
      us[t][cm] = t < n ? u : 0.f;
      if (t < n && ct * 16 + cm < Dv) W.u[(long long)(r0 + t) * P.ld_gate + h * Dv + ct * 16 + cm] = u;
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < TJ; ++j) {
      const bool dok = 16 * (wv + 4 * j) + m < D;
#pragma unroll
      for (int i = 0; i < 4; ++i) S[j][i] *= __builtin_amdgcn_exp2f(cur.el[j][i] * 1.44269504088896341f);
#pragma unroll
      for (int kk = 0; kk < 8; ++kk)
        S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(dok ? cur.kd[j][kk] : 0.f, us[4 * kk + q4][m], S[j], 0, 0, 0);
    }
    ++c;
    r0 = r0n;
    n = nn;
    flags = fn;
    r0n = r0m;
    nn = nm;
    fn = fm;
    return last;
  };
  while (!step(opa, opb) && !step(opb, opa)) {
  }
#pragma unroll
  for (int j = 0; j < TJ; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * (wv + 4 * j) + 4 * q4 + i;
      if (cok && d < D) S0[(long long)d * Dv + col] = S[j][i];
    }
}

static inline size_t delta_out_lds(int D, int Dv) {
  const int Dp = (D + 15) / 16 * 16;
  return (size_t)(DC * (Dp + 4) + DC * (DC + 4) + DC * (Dv + 1)) * sizeof(float);
}
template <typename T, bool HD>
__global__ __launch_bounds__(256) void delta_out_kernel(DeltaParams P, DeltaChunkWs W) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int r0 = W.chunks[4 * c], n = W.chunks[4 * c + 1];
  const int D = P.D, Dv = P.Dv, hg = h / (P.H / P.G), Dp = (D + 15) / 16 * 16, LQ = Dp + 4, V1 = Dv + 1;
  constexpr int LB = DC + 4;
  float* qd = lds;             // [DC][Dp + 4]
  float* Bs = qd + DC * LQ;    // [DC][DC + 4]
  float* ob = Bs + DC * LB;    // [DC][Dv + 1]
  for (int i = tid; i < DC * Dp; i += 256) {
    const int t = i / Dp, d = i % Dp;
    const long long r = r0 + t;
    qd[t * LQ + d] = (t < n && d < D) ? P.x[r * P.ld_x + hg * D + d] * expf(P.lg[r * P.ld_lg + (HD ? h : h * D + d)]) : 0.f;
  }
  for (int i = tid; i < DC * DC; i += 256) {
    const int t = i / DC, sx = i % DC;
    Bs[t * LB + sx] = t < n ? W.Bm[((long long)(r0 + t) * P.H + h) * DC + sx] : 0.f;
  }
  __syncthreads();
  const float* Sin = W.Sin + (long long)c * W.s_stride + (long long)h * D * Dv;
  const int m = lane & 15, q4 = lane >> 4;
  for (int ct = wv; ct * 16 < Dv; ct += 4) {
    const int col = ct * 16 + m;
    const bool cok = col < Dv;
    f32x4 acc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
    for (int d0 = 0; d0 < Dp; d0 += 16) {
      float b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = d0 + 4 * q4 + i;
        b[i] = (cok && d < D) ? Sin[(long long)d * Dv + col] : 0.f;
      }
#pragma unroll
      for (int mt = 0; mt < 2; ++mt) {
        const f32x4 a = *(const f32x4*)&qd[(16 * mt + m) * LQ + d0 + 4 * q4];
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[mt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], acc[mt], 0, 0, 0);
      }
    }
#pragma unroll
    for (int s0 = 0; s0 < DC; s0 += 16) {
      float b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int sx = s0 + 4 * q4 + i;
        b[i] = (cok && sx < n) ? W.u[(long long)(r0 + sx) * P.ld_gate + h * Dv + col] : 0.f;
      }
#pragma unroll
      for (int mt = 0; mt < 2; ++mt) {
        const f32x4 a = *(const f32x4*)&Bs[(16 * mt + m) * LB + s0 + 4 * q4];
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[mt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], acc[mt], 0, 0, 0);
      }
    }
    if (cok) {
#pragma unroll
      for (int mt = 0; mt < 2; ++mt)
#pragma unroll
        for (int i = 0; i < 4; ++i) ob[(16 * mt + 4 * q4 + i) * V1 + col] = acc[mt][i];
    }
  }
  __syncthreads();
  for (int t = wv; t < n; t += 4) {  // a wave per row: the head's RMS norm, its weight, the gate
    float ss = 0.f;
    for (int d = lane; d < Dv; d += 64) ss += ob[t * V1 + d] * ob[t * V1 + d];
    const float f = P.out_scale / sqrtf(wave_sum(ss) / (float)Dv + P.eps);
    for (int d = lane; d < Dv; d += 64)
      st((T*)P.out + (long long)(r0 + t) * P.ld_out + h * Dv + d,
         ob[t * V1 + d] * f * P.norm_w[d] * delta_gate<HD>(P, r0 + t, h * Dv + d));
  }
}
template <bool HD>
static void launch_delta_chunked(const DeltaParams& P, const DeltaChunkWs& W, hipStream_t s) {
  const dim3 grid(W.nchunks, P.H);
  hipLaunchKernelGGL(delta_wy_kernel<HD>, grid, dim3(std::max(256, (P.D + P.Dv + 63) / 64 * 64)), delta_wy_lds(P.D, P.Dv), s, P, W);
  launched("delta_wy");
  const dim3 sg(P.H * ((P.Dv + 15) / 16), W.nchunks);
  const int vec = P.D % 4 == 0 && W.ld_w % 4 == 0 && ((uintptr_t)W.W & 15) == 0;
  if (P.D <= 64 && vec)
    hipLaunchKernelGGL((delta_scan_kernel<1, true, HD>), sg, dim3(256), 0, s, P, W);
  else if (P.D <= 64)
    hipLaunchKernelGGL((delta_scan_kernel<1, false, HD>), sg, dim3(256), 0, s, P, W);
  else if (vec)
    hipLaunchKernelGGL((delta_scan_kernel<2, true, HD>), sg, dim3(256), 0, s, P, W);
  else
    hipLaunchKernelGGL((delta_scan_kernel<2, false, HD>), sg, dim3(256), 0, s, P, W);
  launched("delta_scan");
  if (P.f32)
    hipLaunchKernelGGL((delta_out_kernel<float, HD>), grid, dim3(256), delta_out_lds(P.D, P.Dv), s, P, W);
  else
    hipLaunchKernelGGL((delta_out_kernel<bf16, HD>), grid, dim3(256), delta_out_lds(P.D, P.Dv), s, P, W);
  launched("delta_out");
}
void delta_chunked(const DeltaParams& P, const StepRows& R, const DeltaChunkWs& W, hipStream_t s) {
  check_delta(P, R);
  check(delta_chunk_supported(P.D, P.Dv) && W.chunks && W.nchunks > 0 && W.nchunks <= W.max_chunks && W.Sin && W.W && W.Kd && W.u && W.Bm &&
            W.s_stride >= (long long)P.H * P.D * P.Dv && W.ld_w >= P.H * P.D,
        "chunked gated delta rule: operands (key size <= 128)");
  if (P.head_decay)
    launch_delta_chunked<true>(P, W, s);
  else
    launch_delta_chunked<false>(P, W, s);
}

}  // namespace stack
}  // namespace omx
