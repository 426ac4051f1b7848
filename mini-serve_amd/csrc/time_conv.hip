// A short causal convolution over time on every channel of some columns of a float32 projection, with a bias and an
// optional SiLU:
//     y_t[c] = act(bias[c] + sum_j w[j][c] u_(t - taps + 1 + j)[c]),   u = x[:, col + c] + in_bias[c]
// where u is zero before the sequence's start. Positions of this step come from x; earlier ones from the request's state,
// which holds its last taps - 1 inputs (in_bias included): state[slot][k] is position starts - (taps - 1) + k. All float32;
// the weights come transposed, [taps, C], so that neighbouring channels' lie side by side.
#include "common.h"

struct TimeConvArgs {
  const float* x;  // its first column is the convolution's
  int ld, C, taps;
  const float* w;
  const float* bias;
  const float* in_bias;
  float* out;  // [tokens, C]
  float* state;
  const int* state_slots;
  const int* token_row;
  const int* row_start;
  const int* starts;
  int tokens, act;
};

template <int VEC> struct alignas(4 * VEC) Channels { float e[VEC]; };

// A thread owns VEC channels of a run of `run` consecutive tokens and slides a window of the last taps - 1 inputs along
// them. The first taps - 1 tokens of a request's row in this step are the ones that read its state: whoever has the row's
// first token takes all of them, also those behind its run (and the run they fall into leaves them out), and then writes
// the state as it is after the step. One thread reads and writes a state element, so no other kernel is needed for that.
template <int TAPS, int VEC>
__global__ __launch_bounds__(256) void time_conv_kernel(TimeConvArgs a, int run) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * VEC;
  if (c >= a.C) return;
  typedef Channels<VEC> V;
  constexpr int OLD = TAPS - 1;
  float w[TAPS][VEC], bias[VEC], in[VEC];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) {
    const V v = *reinterpret_cast<const V*>(a.w + (size_t)j * a.C + c);
#pragma unroll
    for (int i = 0; i < VEC; ++i) w[j][i] = v.e[i];
  }
#pragma unroll
  for (int i = 0; i < VEC; ++i) {
    bias[i] = a.bias ? a.bias[c + i] : 0.f;
    in[i] = a.in_bias ? a.in_bias[c + i] : 0.f;
  }
  auto load_x = [&](int t, float* u) {
    const V v = *reinterpret_cast<const V*>(a.x + (size_t)t * a.ld + c);
#pragma unroll
    for (int i = 0; i < VEC; ++i) u[i] = v.e[i] + in[i];
  };
  const int t0 = blockIdx.x * run, t_end = min(t0 + run, a.tokens);
  float win[OLD > 0 ? OLD : 1][VEC];  // win[OLD - 1] is the previous token's input
  int row = -1, first = 0, start = 0;
  float* st = nullptr;
  for (int t = t0; t < a.tokens; ++t) {
    const int b = a.token_row[t];
    const int f = a.row_start[b];
    if (t >= t_end && (f < t0 || f >= t_end || t - f >= OLD)) break;  // past the run: only the leading tokens of a row that began in it
    if (f < t0 && t - f < OLD) continue;                // left to the run that has the row's first token
    if (b != row) {
      row = b, first = f, start = a.starts[b];
      st = OLD > 0 ? a.state + (size_t)a.state_slots[b] * OLD * a.C : nullptr;
#pragma unroll
      for (int j = 0; j < OLD; ++j) {
        const int li = t - first - OLD + j;  // the entry's place in the row; negative: before this step
#pragma unroll
        for (int i = 0; i < VEC; ++i) win[j][i] = 0.f;
        if (li >= 0) {
          load_x(first + li, win[j]);
        } else if (start + li >= 0) {
          const V v = *reinterpret_cast<const V*>(st + (size_t)(OLD + li) * a.C + c);
#pragma unroll
          for (int i = 0; i < VEC; ++i) win[j][i] = v.e[i];
        }
      }
      if (OLD > 0 && t == first) {
        const int n = a.row_start[b + 1] - first;
#pragma unroll
        for (int k = 0; k < OLD; ++k) {
          const int li = n - OLD + k;
          V v;
          if (li >= 0) {
            load_x(first + li, v.e);
          } else {  // the step is shorter than the state: entry k + n moves down
#pragma unroll
            for (int i = 0; i < VEC; ++i) v.e[i] = 0.f;
#pragma unroll
            for (int j = 0; j < OLD; ++j)
              if (j == k + n)
#pragma unroll
                for (int i = 0; i < VEC; ++i) v.e[i] = win[j][i];
          }
          *reinterpret_cast<V*>(st + (size_t)k * a.C + c) = v;
        }
      }
    }
    float u[VEC];
    load_x(t, u);
    V y;
#pragma unroll
    for (int i = 0; i < VEC; ++i) {
      float acc = bias[i];
#pragma unroll
      for (int j = 0; j < OLD; ++j) acc = fmaf(w[j][i], win[j][i], acc);
      acc = fmaf(w[OLD][i], u[i], acc);
      y.e[i] = a.act ? acc / (1.f + expf(-acc)) : acc;
    }
    *reinterpret_cast<V*>(a.out + (size_t)t * a.C + c) = y;
#pragma unroll
    for (int j = 0; j + 1 < OLD; ++j)
#pragma unroll
      for (int i = 0; i < VEC; ++i) win[j][i] = win[j + 1][i];
    if (OLD > 0)
#pragma unroll
      for (int i = 0; i < VEC; ++i) win[OLD - 1][i] = u[i];
  }
}

// Any number of taps: every token reads its inputs where they lie, and a second kernel brings the state up to date.
__global__ __launch_bounds__(256) void time_conv_any_kernel(TimeConvArgs a) {
  const int c = blockIdx.y * 256 + threadIdx.x, t = blockIdx.x;
  if (c >= a.C) return;
  const int b = a.token_row[t], first = a.row_start[b], start = a.starts[b];
  const float* st = a.state + (size_t)a.state_slots[b] * (a.taps - 1) * a.C;
  const float in = a.in_bias ? a.in_bias[c] : 0.f;
  float acc = a.bias ? a.bias[c] : 0.f;
  for (int j = 0; j < a.taps; ++j) {
    const int li = t - first - (a.taps - 1) + j;
    float u = 0.f;
    if (li >= 0) u = a.x[(size_t)(first + li) * a.ld + c] + in;
    else if (start + li >= 0) u = st[(size_t)(a.taps - 1 + li) * a.C + c];
    acc = fmaf(a.w[(size_t)j * a.C + c], u, acc);
  }
  a.out[(size_t)t * a.C + c] = a.act ? acc / (1.f + expf(-acc)) : acc;
}

// A thread owns one channel of one request and walks its taps - 1 entries upwards: an entry that stays moves down from a
// higher index, which has not been written yet.
__global__ __launch_bounds__(256) void time_conv_state_kernel(TimeConvArgs a) {
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
  if (c >= a.C) return;
  const int first = a.row_start[b], n = a.row_start[b + 1] - first, start = a.starts[b];
  float* st = a.state + (size_t)a.state_slots[b] * (a.taps - 1) * a.C;
  const float in = a.in_bias ? a.in_bias[c] : 0.f;
  for (int k = 0; k < a.taps - 1; ++k) {
    const int li = n - (a.taps - 1) + k;
    float u = 0.f;
    if (li >= 0) u = a.x[(size_t)(first + li) * a.ld + c] + in;
    else if (start + li >= 0) u = st[(size_t)(k + n) * a.C + c];
    st[(size_t)k * a.C + c] = u;
  }
}

extern "C" int ms_time_conv(const float* x, int ld, int C, int taps, const float* w, const float* bias, const float* in_bias,
                            float* out, float* state, const int* state_slots, const int* token_row, const int* row_start,
                            const int* starts, int tokens, int rows, int act, hipStream_t st) {
  if (tokens <= 0) return MS_OK;
  if (x == nullptr || C <= 0 || ld < C || taps < 1 || w == nullptr || out == nullptr || (taps > 1 && state == nullptr) ||
      state_slots == nullptr || token_row == nullptr || row_start == nullptr || starts == nullptr || rows <= 0 || rows > 65535 ||
      (act != 0 && act != 1))
    return MS_BAD_ARG;
  TimeConvArgs a{x, ld, C, taps, w, bias, in_bias, out, state, state_slots, token_row, row_start, starts, tokens, act};
  if (taps > 8) {
    if ((C + 255) / 256 > 65535) return MS_UNSUPPORTED;
    time_conv_any_kernel<<<dim3(tokens, (C + 255) / 256), 256, 0, st>>>(a);
    time_conv_state_kernel<<<dim3((C + 255) / 256, rows), 256, 0, st>>>(a);
    return launch_status();
  }
  const bool vec = C % 4 == 0 && ld % 4 == 0 && (size_t)x % 16 == 0 && (size_t)out % 16 == 0 && (size_t)w % 16 == 0 &&
                   (state == nullptr || (size_t)state % 16 == 0);
  const int per = 256 * (vec ? 4 : 1);
  const int run = tokens > 512 ? 8 : tokens > 64 ? 4 : 1;
  const dim3 grid((tokens + run - 1) / run, (C + per - 1) / per);
  if (grid.y > 65535) return MS_UNSUPPORTED;
#define TC(T) case T: if (vec) time_conv_kernel<T, 4><<<grid, 256, 0, st>>>(a, run); else time_conv_kernel<T, 1><<<grid, 256, 0, st>>>(a, run); break
  switch (taps) { TC(1); TC(2); TC(3); TC(4); TC(5); TC(6); TC(7); TC(8); }
#undef TC
  return launch_status();
}
