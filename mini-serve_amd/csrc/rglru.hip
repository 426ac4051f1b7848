// A gated linear recurrence per channel (a real-gated linear recurrent unit):
//     r = sigmoid(R_b u + rb),  i = sigmoid(I_b u + ib)      (R_b, I_b: one square matrix per block b of channels)
//     log a = coef * r,   x = sqrt(1 - a^2) i u,   S_t = a S_(t-1) + x_t,   out_t = S_t gelu_tanh(y_t + yb)
// with coef [W] at most zero. u and y are float32, everything between them and `out` is float32, the gates' products
// included: where R and I are bfloat16, u is cut into three bfloat16 pieces that add up to it, whose products with the
// weights are exact and meet in float32 sums on the matrix cores; where they are float32 the matrix cores' float32
// instruction takes both as they are.
// A step of single tokens is one kernel, gates and recurrence together. Other steps write a and x and then run the
// recurrence: rows of few tokens are walked, rows of many in chunks of LRU_CHUNK tokens and three passes (a chunk's product
// of a and its own state from zero; chunk after chunk the state before each; every chunk's outputs from there).
#include "common.h"

#define LRU_CHUNK 32
#define LRU_TWO_RUNS_FROM 512  // blocks

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 lru_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float lru_floatx4;

struct LruArgs {
  const float* u;  // [T, W]
  int T, W, bs;    // bs: channels of a block
  const void* R;   // [W / bs, bs, bs] (out, in)
  const void* I;
  const float* rb;    // [W]
  const float* ib;    // [W]
  const float* coef;  // [W]
  float2* ax;         // [T, W]: a and x side by side
  const float* y;     // [T, ldy]
  int ldy;
  const float* yb;  // [W]
  void* out;        // [T, W]
  int out_bf16;
  float* S;  // [slots, W]
  const int* row_start;
  const int* starts;
  const int* state_slots;
  int rows;
  float* sum;  // [chunks, 2, W]: a chunk's product of a, and its state from zero, later the state before it
};

__device__ __forceinline__ void lru_store(const LruArgs& p, int t, int c, float S) {
  const float v = S * activate(p.y[(size_t)t * p.ldy + c] + p.yb[c], MS_ACT_GELU_TANH);
  const size_t at = (size_t)t * p.W + c;
  if (p.out_bf16) ((bf16*)p.out)[at] = static_cast<bf16>(v);
  else ((float*)p.out)[at] = v;
}

// The hardware's exponential and reciprocal, each good to a unit in the last place or so.
__device__ __forceinline__ float lru_sigmoid(float z) { return __builtin_amdgcn_rcpf(1.f + __expf(-z)); }

// 1 - exp(y) for y <= 0: near zero by its series, where the difference would lose what it is made of.
__device__ __forceinline__ float lru_one_minus_exp(float y, float exp_y) {
  float s = 1.f / 5040.f;
  s = fmaf(s, y, 1.f / 720.f);
  s = fmaf(s, y, 1.f / 120.f);
  s = fmaf(s, y, 1.f / 24.f);
  s = fmaf(s, y, 1.f / 6.f);
  s = fmaf(s, y, 0.5f);
  s = fmaf(s, y, 1.f);
  return y > -0.25f ? -y * s : 1.f - exp_y;
}

struct LruChannel { float rb, ib, coef; };
__device__ __forceinline__ LruChannel lru_channel(const LruArgs& p, int c) { return LruChannel{p.rb[c], p.ib[c], p.coef[c]}; }

// What the two gates' sums make of channel c of token t, whose input is u. STEP: row t of the step is token t alone.
template <bool STEP> __device__ __forceinline__ void lru_finish(const LruArgs& p, const LruChannel& ch, int t, int c, float u, float rs, float is) {
  const float r = lru_sigmoid(rs + ch.rb), i = lru_sigmoid(is + ch.ib);
  const float la = ch.coef * r;
  const float a = expf(la), x = __builtin_amdgcn_sqrtf(lru_one_minus_exp(2.f * la, a * a)) * (i * u);
  if (STEP) {
    float* s = p.S + (size_t)p.state_slots[t] * p.W + c;
    const float S = (p.starts[t] == 0 ? 0.f : a * *s) + x;
    *s = S;
    lru_store(p, t, c, S);
  } else {
    p.ax[(size_t)t * p.W + c] = make_float2(a, x);
  }
}

// Eight consecutive elements from p + k, those of u at or past K zero (what a weight is there does not matter then). ALIGNED:
// all eight lie inside K or none does; loads past it go to the last eight instead of being left out, so that nothing branches.
template <bool ALIGNED> __device__ __forceinline__ void lru_load8(const float* p, int k, int K, bool ok, float* v) {
  if (ALIGNED) {
    const float* q = p + max(min(k, K - 8), 0);
    const float4 lo = *reinterpret_cast<const float4*>(q), hi = *reinterpret_cast<const float4*>(q + 4);
    const bool in = k < K;
    v[0] = in ? lo.x : 0.f; v[1] = in ? lo.y : 0.f; v[2] = in ? lo.z : 0.f; v[3] = in ? lo.w : 0.f;
    v[4] = in ? hi.x : 0.f; v[5] = in ? hi.y : 0.f; v[6] = in ? hi.z : 0.f; v[7] = in ? hi.w : 0.f;
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = (ok && k + e < K) ? p[k + e] : 0.f;
  }
}
template <bool ALIGNED> __device__ __forceinline__ lru_bf16x8 lru_load8(const bf16* p, int k, int K, bool ok) {
  union { uint4 u; lru_bf16x8 v; bf16 e[8]; } x;
  x.u = make_uint4(0, 0, 0, 0);
  if (ALIGNED) {
    x.u = *reinterpret_cast<const uint4*>(p + max(min(k, K - 8), 0));
  } else if (ok) {
#pragma unroll
    for (int e = 0; e < 8; ++e)
      if (k + e < K) x.e[e] = p[k + e];
  }
  return x.v;
}

// A block owns the gates of 64 channels of one block of channels for 64 MT tokens (a wave 16 MT of them) or, NT = 1 (steps of few
// tokens), of 16 channels for 16 tokens, its waves sharing k: their sums meet in LDS and are added in wave order. Operands
// straight from memory, those of the next 32 k asked for before the products of these: the weights of a block of channels are
// small and stay in the cache.
template <bool STEP, int NT, int MT, bool ALIGNED>
__global__ __launch_bounds__(256) void lru_gates_bf16_kernel(LruArgs p) {
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, l16 = lane % 16, grp = lane / 16;
  const int b = blockIdx.z, K = p.bs;
  const int m0 = NT == 1 ? blockIdx.x * 16 : (blockIdx.x * 4 + wave) * 16 * MT;
  const int n0 = blockIdx.y * (16 * NT);
  if (m0 >= p.T || n0 >= K) return;
  const int k_quarter = ((K + 3) / 4 + 31) / 32 * 32;
  const int k_lo = NT == 1 ? min(K, wave * k_quarter) : 0, k_hi = NT == 1 ? min(K, k_lo + k_quarter) : K;
  const float* up[MT];
  bool row_ok[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    row_ok[mt] = m0 + mt * 16 + l16 < p.T;
    up[mt] = p.u + (size_t)(row_ok[mt] ? m0 + mt * 16 + l16 : 0) * p.W + (size_t)b * K;
  }
  const bf16 *rp[NT], *ip[NT];
  bool col_ok[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) {
    col_ok[nt] = n0 + nt * 16 + l16 < K;
    const size_t at = ((size_t)b * K + (col_ok[nt] ? n0 + nt * 16 + l16 : 0)) * K;
    rp[nt] = (const bf16*)p.R + at;
    ip[nt] = (const bf16*)p.I + at;
  }
  lru_floatx4 accr[MT][NT], acci[MT][NT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt)
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) accr[mt][nt] = acci[mt][nt] = lru_floatx4{0.f, 0.f, 0.f, 0.f};
  float v[MT][8];
  lru_bf16x8 rw[NT], iw[NT];
  auto load = [&](int k) __attribute__((always_inline)) {
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) lru_load8<ALIGNED>(up[mt], k, k_hi, row_ok[mt], v[mt]);
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      rw[nt] = lru_load8<ALIGNED>(rp[nt], k, k_hi, col_ok[nt]);
      iw[nt] = lru_load8<ALIGNED>(ip[nt], k, k_hi, col_ok[nt]);
    }
  };
  load(k_lo + grp * 8);
  for (int k0 = k_lo; k0 < k_hi; k0 += 32) {
    union { lru_bf16x8 v; bf16 e[8]; } piece[MT][3];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        piece[mt][0].e[e] = static_cast<bf16>(v[mt][e]);
        const float rest = v[mt][e] - to_f32(piece[mt][0].e[e]);
        piece[mt][1].e[e] = static_cast<bf16>(rest);
        piece[mt][2].e[e] = static_cast<bf16>(rest - to_f32(piece[mt][1].e[e]));
      }
    lru_bf16x8 rn[NT], in[NT];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) rn[nt] = rw[nt], in[nt] = iw[nt];
    load(k0 + 32 + grp * 8);  // (past the end: zeros)
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
#pragma unroll
      for (int s = 2; s >= 0; --s)  // the smallest piece first
#pragma unroll
        for (int mt = 0; mt < MT; ++mt) {
          accr[mt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(piece[mt][s].v, rn[nt], accr[mt][nt], 0, 0, 0);
          acci[mt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(piece[mt][s].v, in[nt], acci[mt][nt], 0, 0, 0);
        }
  }
  if constexpr (NT == 1) {
    static_assert(MT == 1, "one run of tokens");
    __shared__ float meet[4][2][4][WAVE];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      meet[wave][0][r][lane] = accr[0][0][r];
      meet[wave][1][r][lane] = acci[0][0][r];
    }
    __syncthreads();
    float s[2] = {0.f, 0.f};  // wave r finishes the tile's rows r, r + 4, ...
#pragma unroll
    for (int g = 0; g < 2; ++g)
#pragma unroll
      for (int w = 0; w < 4; ++w) s[g] += meet[w][g][wave][lane];
    const int t = m0 + grp * 4 + wave;
    const int c = b * K + n0 + l16;
    if (t < p.T && col_ok[0]) lru_finish<STEP>(p, lru_channel(p, c), t, c, p.u[(size_t)t * p.W + c], s[0], s[1]);
    return;
  }
  // what the tile's elements need is asked for at once: behind the first store the loads would go one by one
  LruChannel ch[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) ch[nt] = lru_channel(p, b * K + min(n0 + nt * 16 + l16, K - 1));
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    float u[4][NT];
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
        u[r][nt] = p.u[(size_t)min(m0 + mt * 16 + grp * 4 + r, p.T - 1) * p.W + b * K + min(n0 + nt * 16 + l16, K - 1)];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = m0 + mt * 16 + grp * 4 + r;
      if (t >= p.T) continue;
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
        if (col_ok[nt]) lru_finish<STEP>(p, ch[nt], t, b * K + n0 + nt * 16 + l16, u[r][nt], accr[mt][nt][r], acci[mt][nt][r]);
    }
  }
}

// The same with float32 weights: of each 16 consecutive k a lane holds four, one per instruction.
template <bool STEP, int NT, int MT, bool ALIGNED>
__global__ __launch_bounds__(256) void lru_gates_f32_kernel(LruArgs p) {
  const int lane = threadIdx.x % WAVE, wave = threadIdx.x / WAVE, l16 = lane % 16, grp = lane / 16;
  const int b = blockIdx.z, K = p.bs;
  const int m0 = NT == 1 ? blockIdx.x * 16 : blockIdx.x * 64 + wave * 16;
  const int n0 = blockIdx.y * 64 + (NT == 1 ? wave * 16 : 0);
  if (m0 >= p.T || n0 >= K) return;
  const bool row_ok = m0 + l16 < p.T;
  const float* up = p.u + (size_t)(row_ok ? m0 + l16 : 0) * p.W + (size_t)b * K;
  lru_floatx4 accr[NT], acci[NT];
#pragma unroll
  for (int nt = 0; nt < NT; ++nt) accr[nt] = acci[nt] = lru_floatx4{0.f, 0.f, 0.f, 0.f};
  auto load4 = [&](const float* q, int k, bool ok, float* v) __attribute__((always_inline)) {
    if (ALIGNED) {
      const float4 w = ok && k < K ? *reinterpret_cast<const float4*>(q + k) : make_float4(0.f, 0.f, 0.f, 0.f);
      v[0] = w.x; v[1] = w.y; v[2] = w.z; v[3] = w.w;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = (ok && k + e < K) ? q[k + e] : 0.f;
    }
  };
  for (int k0 = 0; k0 < K; k0 += 16) {
    const int k = k0 + grp * 4;
    float uv[4];
    load4(up, k, row_ok, uv);
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const bool ok = n0 + nt * 16 + l16 < K;
      const size_t at = ((size_t)b * K + (ok ? n0 + nt * 16 + l16 : 0)) * K;
      float rw[4], iw[4];
      load4((const float*)p.R + at, k, ok, rw);
      load4((const float*)p.I + at, k, ok, iw);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        accr[nt] = __builtin_amdgcn_mfma_f32_16x16x4f32(uv[e], rw[e], accr[nt], 0, 0, 0);
        acci[nt] = __builtin_amdgcn_mfma_f32_16x16x4f32(uv[e], iw[e], acci[nt], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = m0 + grp * 4 + r;
    if (t >= p.T) continue;
#pragma unroll
    for (int nt = 0; nt < NT; ++nt)
      if (n0 + nt * 16 + l16 < K) {
        const int c = b * K + n0 + nt * 16 + l16;
        lru_finish<STEP>(p, lru_channel(p, c), t, c, p.u[(size_t)t * p.W + c], accr[nt][r], acci[nt][r]);
      }
  }
}

// A thread owns one channel of one row and walks its tokens from the slot's state.
__global__ __launch_bounds__(256) void lru_walk_kernel(LruArgs p) {
  const int c = blockIdx.y * 256 + threadIdx.x, b = blockIdx.x;
  if (c >= p.W) return;
  float* s = p.S + (size_t)p.state_slots[b] * p.W + c;
  float S = p.starts[b] == 0 ? 0.f : *s;
  for (int t = p.row_start[b]; t < p.row_start[b + 1]; ++t) {
    const float2 ax = p.ax[(size_t)t * p.W + c];
    S = ax.x * S + ax.y;
    lru_store(p, t, c, S);
  }
  *s = S;
}

// The chunk `c` of the step: its first token and token count.
__device__ __forceinline__ void lru_find_chunk(const int* __restrict__ row_start, int rows, int c, int* first, int* count) {
  int b = 0, at = 0;
  for (; b < rows - 1; ++b) {
    const int nc = (row_start[b + 1] - row_start[b] + LRU_CHUNK - 1) / LRU_CHUNK;
    if (c < at + nc) break;
    at += nc;
  }
  *first = row_start[b] + (c - at) * LRU_CHUNK;
  const int left = row_start[b + 1] - *first;
  *count = left < LRU_CHUNK ? left : LRU_CHUNK;
}

// A chunk's tokens one after the other for channel c, eight tokens' a and x asked for at a time: step(t, a, x).
template <typename F> __device__ __forceinline__ void lru_chunk(const LruArgs& p, int c, int first, int count, F step) {
  constexpr int AHEAD = 8;
  for (int k0 = 0; k0 < count; k0 += AHEAD) {
    float2 v[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) v[i] = p.ax[(size_t)(first + min(k0 + i, count - 1)) * p.W + c];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i)
      if (k0 + i < count) step(first + k0 + i, v[i].x, v[i].y);
  }
}

__global__ __launch_bounds__(256) void lru_chunk_summary_kernel(LruArgs p) {
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= p.W) return;
  int first, count;
  lru_find_chunk(p.row_start, p.rows, blockIdx.x, &first, &count);
  float prod = 1.f, S = 0.f;
  lru_chunk(p, c, first, count, [&](int, float a, float x) {
    prod *= a;
    S = a * S + x;
  });
  p.sum[(size_t)blockIdx.x * 2 * p.W + c] = prod;
  p.sum[((size_t)blockIdx.x * 2 + 1) * p.W + c] = S;
}

__global__ __launch_bounds__(64) void lru_chunk_scan_kernel(LruArgs p) {
  const int c = blockIdx.x * 64 + threadIdx.x, b = blockIdx.y;
  if (c >= p.W) return;
  int base = 0;
  for (int r = 0; r < b; ++r) base += (p.row_start[r + 1] - p.row_start[r] + LRU_CHUNK - 1) / LRU_CHUNK;
  const int nc = (p.row_start[b + 1] - p.row_start[b] + LRU_CHUNK - 1) / LRU_CHUNK;
  float* s = p.S + (size_t)p.state_slots[b] * p.W + c;
  float S = p.starts[b] == 0 ? 0.f : *s;
  constexpr int AHEAD = 16;
  for (int k0 = 0; k0 < nc; k0 += AHEAD) {
    float a[AHEAD], x[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const size_t at = (size_t)(base + min(k0 + i, nc - 1)) * 2 * p.W + c;
      a[i] = p.sum[at];
      x[i] = p.sum[at + p.W];
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      if (k0 + i >= nc) break;
      p.sum[((size_t)(base + k0 + i) * 2 + 1) * p.W + c] = S;
      S = a[i] * S + x[i];
    }
  }
  *s = S;
}

__global__ __launch_bounds__(256) void lru_chunk_output_kernel(LruArgs p) {
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= p.W) return;
  int first, count;
  lru_find_chunk(p.row_start, p.rows, blockIdx.x, &first, &count);
  float S = p.sum[((size_t)blockIdx.x * 2 + 1) * p.W + c];
  lru_chunk(p, c, first, count, [&](int t, float a, float x) {
    S = a * S + x;
    lru_store(p, t, c, S);
  });
}

extern "C" int ms_rglru_chunk_tokens() { return LRU_CHUNK; }

// u [T, W]; R, I [blocks, W / blocks, W / blocks]; y's column c of token t is y[t ldy + c]. form 0: every row is one token (ax,
// sum unused); 1: rows are walked (ax [T, W, 2] scratch); 2: rows in chunks, `chunks` = sum over the rows of ceil(tokens /
// LRU_CHUNK), sum [chunks, 2, W] scratch.
extern "C" int ms_rglru(const float* u, int T, int W, int blocks, const void* R, const void* I, int w_is_bf16, const float* rb,
                        const float* ib, const float* coef, float* ax, const float* y, int ldy, const float* yb, void* out,
                        int out_bf16, float* S, const int* row_start, const int* starts, const int* state_slots, int rows, int form,
                        int chunks, float* sum, hipStream_t st) {
  if (T <= 0 || rows <= 0) return MS_OK;
  if (W <= 0 || blocks <= 0 || W % blocks || u == nullptr || R == nullptr || I == nullptr || rb == nullptr || ib == nullptr ||
      coef == nullptr || y == nullptr || ldy < W || yb == nullptr || out == nullptr || S == nullptr || row_start == nullptr ||
      starts == nullptr || state_slots == nullptr || form < 0 || form > 2 || (form == 0 && rows != T) ||
      (form > 0 && (ax == nullptr || (size_t)ax % 8)) || (form == 2 && (sum == nullptr || chunks <= 0)))
    return MS_BAD_ARG;
  const int bs = W / blocks;
  if (blocks > 65535 || (W + 255) / 256 > 65535 || rows > 65535) return MS_UNSUPPORTED;
  LruArgs p{u, T, W, bs, R, I, rb, ib, coef, (float2*)ax, y, ldy, yb, out, out_bf16, S, row_start, starts, state_slots, rows, sum};
  const bool few = T <= 64;
  // two runs of 16 tokens a wave halve how often the weights are read, where that leaves blocks enough
  const int mt = w_is_bf16 && (long)((T + 127) / 128) * ((bs + 63) / 64) * blocks >= LRU_TWO_RUNS_FROM ? 2 : 1;
  const int cols_of_block = few && w_is_bf16 ? 16 : 64;
  const dim3 grid(few ? (T + 15) / 16 : (T + 64 * mt - 1) / (64 * mt), (bs + cols_of_block - 1) / cols_of_block, blocks);
  if (grid.y > 65535) return MS_UNSUPPORTED;
  const bool aligned = bs % 8 == 0 && (size_t)u % 16 == 0 && (size_t)R % 16 == 0 && (size_t)I % 16 == 0;
#define LRU_GATES(F, S_, N, M)                                                      \
  do {                                                                              \
    if (aligned) lru_gates_##F##_kernel<S_, N, M, true><<<grid, 256, 0, st>>>(p);   \
    else lru_gates_##F##_kernel<S_, N, M, false><<<grid, 256, 0, st>>>(p);          \
  } while (0)
#define LRU_FORM(F, M)                                                                    \
  do {                                                                                    \
    if (form == 0) { if (few) LRU_GATES(F, true, 1, 1); else LRU_GATES(F, true, 4, M); }  \
    else { if (few) LRU_GATES(F, false, 1, 1); else LRU_GATES(F, false, 4, M); }          \
  } while (0)
  if (w_is_bf16) { if (mt == 2) LRU_FORM(bf16, 2); else LRU_FORM(bf16, 1); }
  else LRU_FORM(f32, 1);
#undef LRU_FORM
#undef LRU_GATES
  const unsigned cols = (unsigned)((W + 255) / 256);
  if (form == 1) {
    lru_walk_kernel<<<dim3(rows, cols), 256, 0, st>>>(p);
  } else if (form == 2) {
    lru_chunk_summary_kernel<<<dim3(chunks, cols), 256, 0, st>>>(p);
    lru_chunk_scan_kernel<<<dim3((W + 63) / 64, rows), 64, 0, st>>>(p);
    lru_chunk_output_kernel<<<dim3(chunks, cols), 256, 0, st>>>(p);
  }
  return launch_status();
}
