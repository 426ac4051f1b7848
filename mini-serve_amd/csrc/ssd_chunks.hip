// The step-size recurrence of recurrence.hip (MS_REC_STEP) for rows that bring many tokens, in chunks of SSD_CHUNK tokens
// and three passes:
//     S_t = exp(decay d_t) S_(t-1) + d_t k_t v_t^T,   o_t = S_t^T q_t + skip v_t       (S: [D, E]; k, q: [D]; v: [E])
// with L_t the sum of decay * d through t from the chunk's start (every exponent below is at most zero, decay being negative):
//   1. per (chunk, head): the chunk's own contribution to the state at its end, U = sum_j exp(L_last - L_j) d_j k_j v_j^T;
//   2. per (row, head), chunk after chunk: S' = exp(L_last) S + U; the state *before* each chunk takes U's place, the state
//      after the last one goes to the request's slot;
//   3. per (chunk, head): o_t = exp(L_t) S0^T q_t + sum_(j <= t) (q_t . k_j) exp(L_t - L_j) d_j v_j + skip v_t.
// The products run on the matrix cores in true float32 (v_mfma_f32_16x16x4_f32: float32 operands and sums). The running sums
// are double precision: the kernels need their differences, which may be small where the sums are in the hundreds.
// A lane's operand element is row (or column) lane % 16 and, of each 16 consecutive k, those from 4 (lane / 16) on, one per
// instruction: the same cut for both operands, so that four instructions cover the 16 and a lane reads them as one vector
// where k runs along a row.
#include "common.h"

#define SSD_CHUNK 64
#define SSD_MAX_DIM 256

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float ssd_floatx4;

struct SsdArgs {
  const float* x;  // [tokens, ld]: q, k ([groups, D] each) and v ([H, E]) in columns
  int ld, q_off, k_off, v_off;
  int H, D, E, share;
  const float* step;  // [tokens, ld_step], head h's in column h, before bias and softplus
  int ld_step;
  const float* step_bias;
  const float* decay;  // [H], negative
  const float* skip;   // [H]
  float* S;            // [slots, H, D, E]
  const int* row_start;
  const int* starts;
  const int* state_slots;
  float* out;   // [tokens, H E]
  float* U;     // [chunks, H, D E]
  float* total; // [chunks, H]: L_last
  int rows, vec, HB;
};

__device__ __forceinline__ ssd_floatx4 ssd_mfma(float a, float b, ssd_floatx4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// The chunk `c` of the step: its first token and token count.
__device__ __forceinline__ void ssd_find_chunk(const int* __restrict__ row_start, int rows, int c, int* first, int* count) {
  int b = 0, at = 0;
  for (; b < rows - 1; ++b) {
    const int nc = (row_start[b + 1] - row_start[b] + SSD_CHUNK - 1) / SSD_CHUNK;
    if (c < at + nc) break;
    at += nc;
  }
  *first = row_start[b] + (c - at) * SSD_CHUNK;
  const int left = row_start[b + 1] - *first;
  *count = left < SSD_CHUNK ? left : SSD_CHUNK;
}

// One wave, one head: step sizes of the chunk's tokens (zero past its end) into d[], running sums of decay * d into L[].
__device__ __forceinline__ void ssd_steps(const SsdArgs& a, int h, int first, int count, float* d, double* L) {
  const int j = threadIdx.x % WAVE;
  float dj = 0.f;
  if (j < count) dj = softplus(a.step[(size_t)(first + j) * a.ld_step + h] + (a.step_bias ? a.step_bias[h] : 0.f));
  double run = (double)(a.decay[h] * dj);
#pragma unroll
  for (int off = 1; off < WAVE; off <<= 1) {
    const double v = __shfl_up(run, off, WAVE);
    if (j >= off) run += v;
  }
  d[j] = dj;
  L[j] = run;
}

// What a wave of the first and third pass works on. A block owns one chunk and up to four heads that share their keys and
// queries: with HB = 4 (2, 1) heads a block, wave w has head w % HB and every 4 / HB-th run of 16 value columns from w / HB on.
struct SsdWork {
  int group, h, run0, run_step, first, count;
  bool live;
};
__device__ __forceinline__ SsdWork ssd_work(const SsdArgs& a) {
  SsdWork k;
  const int wave = threadIdx.x / WAVE, sets = (a.share + a.HB - 1) / a.HB;
  k.group = blockIdx.y / sets;
  const int in_group = (blockIdx.y % sets) * a.HB + wave % a.HB;
  k.live = in_group < a.share;
  k.h = k.group * a.share + (k.live ? in_group : 0);
  k.run0 = wave / a.HB;
  k.run_step = 4 / a.HB;
  ssd_find_chunk(a.row_start, a.rows, blockIdx.x, &k.first, &k.count);
  return k;
}

// Rows first .. first + count - 1, columns col .. col + n - 1 of x into tile[row][column] (row stride ts); rows past count and
// columns from n to np are zero.
__device__ __forceinline__ void ssd_stage(const SsdArgs& a, int first, int count, int col, int n, int np, float* tile, int ts) {
  if (a.vec) {  // n, the columns' start and the rows' stride are multiples of four
    const int per = np / 4;
    for (int i = threadIdx.x; i < SSD_CHUNK * per; i += 256) {
      const int j = i / per, c = (i % per) * 4;
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      if (j < count && c < n) v = *reinterpret_cast<const float4*>(a.x + (size_t)(first + j) * a.ld + col + c);
      *reinterpret_cast<float4*>(tile + j * ts + c) = v;
    }
  } else {
    for (int i = threadIdx.x; i < SSD_CHUNK * np; i += 256) {
      const int j = i / np, c = i % np;
      tile[j * ts + c] = (j < count && c < n) ? a.x[(size_t)(first + j) * a.ld + col + c] : 0.f;
    }
  }
}

// Pass 1. The keys, which every head of the block reads, are staged in LDS; the values, weighted per token, stay in the
// registers of their wave, four runs of 16 columns at a time.
__global__ __launch_bounds__(256, 2) void ssd_summary_kernel(SsdArgs a) {
  extern __shared__ __attribute__((aligned(16))) float ssd_lds[];
  __shared__ float d[4][SSD_CHUNK];
  __shared__ double L[4][SSD_CHUNK];
  constexpr int KI = SSD_CHUNK / 4, RUNS = 4;  // KI: a lane's tokens, those from 4 (lane / 16) on of every 16
  const SsdWork k = ssd_work(a);
  const int D = a.D, E = a.E, h = k.h, first = k.first, count = k.count, wave = threadIdx.x / WAVE, l16 = threadIdx.x % 16, grp = (threadIdx.x % WAVE) / 16;
  const int DP = (D + 15) & ~15, ks = DP + 4;
  float* K = ssd_lds;  // [SSD_CHUNK][ks]
  const float* vp = a.x + (size_t)first * a.ld + a.v_off + h * E;
  float v[RUNS][KI];
  // Columns past the last are read again and not stored; rows past the chunk's end, whose weights are zero, likewise.
  auto load = [&](int run) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < RUNS; ++u) {
      const unsigned e = (unsigned)min((run + u * k.run_step) * 16 + l16, E - 1);
#pragma unroll
      for (int i = 0; i < KI; ++i) v[u][i] = vp[(unsigned)min((i / 4) * 16 + grp * 4 + i % 4, count - 1) * (unsigned)a.ld + e];
    }
  };
  load(k.run0);
  ssd_stage(a, first, count, a.k_off + k.group * D, D, DP, K, ks);
  ssd_steps(a, h, first, count, d[wave], L[wave]);
  __syncthreads();
  if (!k.live) return;
  const double last = L[wave][SSD_CHUNK - 1];  // (tokens past the end add nothing)
  if (k.run0 == 0 && threadIdx.x % WAVE == 0) a.total[(size_t)blockIdx.x * a.H + h] = (float)last;
  float* Uo = a.U + ((size_t)blockIdx.x * a.H + h) * D * E;
  for (int run = k.run0; run * 16 < E; run += RUNS * k.run_step) {
    if (run != k.run0) load(run);
#pragma unroll
    for (int i = 0; i < KI; ++i) {
      const int j = (i / 4) * 16 + grp * 4 + i % 4;
      const float w = expf((float)(last - L[wave][j])) * d[wave][j];
#pragma unroll
      for (int u = 0; u < RUNS; ++u) v[u][i] *= w;
    }
    for (int n0 = 0; n0 < D; n0 += 16) {
      ssd_floatx4 acc[RUNS];
#pragma unroll
      for (int u = 0; u < RUNS; ++u) acc[u] = ssd_floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < KI; ++i) {
        const float kv = K[((i / 4) * 16 + grp * 4 + i % 4) * ks + n0 + l16];
#pragma unroll
        for (int u = 0; u < RUNS; ++u) acc[u] = ssd_mfma(kv, v[u][i], acc[u]);
      }
#pragma unroll
      for (int u = 0; u < RUNS; ++u) {
        const int e = (run + u * k.run_step) * 16 + l16;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int n = n0 + grp * 4 + r;
          if (n < D && e < E) Uo[(size_t)n * E + e] = acc[u][r];
        }
      }
    }
  }
}

// Pass 2. grid (runs of 256 state elements, H, rows); a thread owns one element and asks for several chunks' at a time.
__global__ __launch_bounds__(256) void ssd_scan_kernel(SsdArgs a) {
  const int h = blockIdx.y, b = blockIdx.z, idx = blockIdx.x * 256 + threadIdx.x;
  const int DE = a.D * a.E;
  if (idx >= DE) return;
  int base = 0;
  for (int r = 0; r < b; ++r) base += (a.row_start[r + 1] - a.row_start[r] + SSD_CHUNK - 1) / SSD_CHUNK;
  const int nc = (a.row_start[b + 1] - a.row_start[b] + SSD_CHUNK - 1) / SSD_CHUNK;
  float* Sg = a.S + ((size_t)a.state_slots[b] * a.H + h) * (size_t)DE + idx;
  float S = a.starts[b] == 0 ? 0.f : *Sg;
  constexpr int AHEAD = 8;
  for (int k0 = 0; k0 < nc; k0 += AHEAD) {
    float u[AHEAD], f[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const size_t at = (size_t)(base + min(k0 + i, nc - 1)) * a.H + h;
      u[i] = a.U[at * DE + idx];
      f[i] = a.total[at];
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      if (k0 + i >= nc) break;
      a.U[((size_t)(base + k0 + i) * a.H + h) * DE + idx] = S;
      S = expf(f[i]) * S + u[i];
    }
  }
  *Sg = S;
}

// Pass 3. The scores q . k of the 16 x 16 tiles on and below the diagonal are formed once for the block's heads (they take
// the keys' place in LDS); from there on every wave works for itself: its head's weights P as operand fragments in registers,
// then, for each of its runs of 16 value columns, the entry state's part and the weighted values'. The fragments of S0 and v
// are read by this wave alone, straight from memory, those of the next run before the products of this one. NK: runs of 16
// elements of a key, D padded to them with zeros.
template <int NK>
__global__ __launch_bounds__(256, NK <= 8 ? 2 : 1) void ssd_output_kernel(SsdArgs a) {
  extern __shared__ __attribute__((aligned(16))) float ssd_lds[];
  __shared__ float d[4][SSD_CHUNK];
  __shared__ double L[4][SSD_CHUNK];
  constexpr int DP = NK * 16, ks = DP + 4, ps = SSD_CHUNK + 4, KI = SSD_CHUNK / 4;
  const SsdWork k = ssd_work(a);
  const int D = a.D, E = a.E, h = k.h, first = k.first, count = k.count, wave = threadIdx.x / WAVE, l16 = threadIdx.x % 16, grp = (threadIdx.x % WAVE) / 16;
  float* Q = ssd_lds;             // [SSD_CHUNK][ks]
  float* K = Q + SSD_CHUNK * ks;  // [SSD_CHUNK][ks], later the scores [SSD_CHUNK][ps]
  float* G = K;
  const float* S0 = a.U + ((size_t)blockIdx.x * a.H + h) * D * E;
  const float* vp = a.x + (size_t)first * a.ld + a.v_off + h * E;
  // What lies past the last row or column is read from the last: it meets zeros (padded queries, masked weights) or is not stored.
  float s0[NK * 4], v[KI];
  auto load = [&](int run) __attribute__((always_inline)) {
    const unsigned e = (unsigned)min(run * 16 + l16, E - 1);
#pragma unroll
    for (int i = 0; i < NK * 4; ++i) s0[i] = S0[(unsigned)min((i / 4) * 16 + grp * 4 + i % 4, D - 1) * (unsigned)E + e];
#pragma unroll
    for (int i = 0; i < KI; ++i) v[i] = vp[(unsigned)min((i / 4) * 16 + grp * 4 + i % 4, count - 1) * (unsigned)a.ld + e];
  };
  load(k.run0);
  ssd_stage(a, first, count, a.q_off + k.group * D, D, DP, Q, ks);
  ssd_stage(a, first, count, a.k_off + k.group * D, D, DP, K, ks);
  ssd_steps(a, h, first, count, d[wave], L[wave]);
  __syncthreads();
  // tile p of the ten on and below the diagonal: (0,0) (1,0) (1,1) (2,0) ...
  ssd_floatx4 sc[3];
#pragma unroll
  for (int u = 0; u < 3; ++u) {
    const int p = wave + 4 * u;
    sc[u] = ssd_floatx4{0.f, 0.f, 0.f, 0.f};
    if (p >= 10) continue;
    const int ti = p >= 6 ? 3 : p >= 3 ? 2 : p >= 1 ? 1 : 0, tj = p - ti * (ti + 1) / 2;
    const float* qr = Q + (ti * 16 + l16) * ks + grp * 4;
    const float* kr = K + (tj * 16 + l16) * ks + grp * 4;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const float4 qv = *reinterpret_cast<const float4*>(qr + i * 16), kv = *reinterpret_cast<const float4*>(kr + i * 16);
      sc[u] = ssd_mfma(qv.x, kv.x, sc[u]);
      sc[u] = ssd_mfma(qv.y, kv.y, sc[u]);
      sc[u] = ssd_mfma(qv.z, kv.z, sc[u]);
      sc[u] = ssd_mfma(qv.w, kv.w, sc[u]);
    }
  }
  __syncthreads();  // every wave is done with the keys
#pragma unroll
  for (int u = 0; u < 3; ++u) {
    const int p = wave + 4 * u;
    if (p >= 10) continue;
    const int ti = p >= 6 ? 3 : p >= 3 ? 2 : p >= 1 ? 1 : 0, tj = p - ti * (ti + 1) / 2;
#pragma unroll
    for (int r = 0; r < 4; ++r) G[(ti * 16 + grp * 4 + r) * ps + tj * 16 + l16] = sc[u][r];
  }
  __syncthreads();
  if (!k.live) return;
  float pf[10][4];  // the weights of tile (ti, tj): row ti 16 + lane % 16, columns tj 16 + 4 (lane / 16) ..
#pragma unroll
  for (int ti = 0; ti < 4; ++ti) {
    const int t = ti * 16 + l16;
    const double Lt = L[wave][t];
#pragma unroll
    for (int tj = 0; tj <= ti; ++tj) {
      const int j = tj * 16 + grp * 4;
      const float4 g = *reinterpret_cast<const float4*>(G + t * ps + j);
      const float gv[4] = {g.x, g.y, g.z, g.w};
#pragma unroll
      for (int c = 0; c < 4; ++c)
        pf[ti * (ti + 1) / 2 + tj][c] = j + c <= t ? gv[c] * expf((float)(Lt - L[wave][j + c])) * d[wave][j + c] : 0.f;
    }
  }
  float eL[4][4];
#pragma unroll
  for (int ti = 0; ti < 4; ++ti)
#pragma unroll
    for (int r = 0; r < 4; ++r) eL[ti][r] = expf((float)L[wave][ti * 16 + grp * 4 + r]);
  const float skip = a.skip[h];
#pragma unroll 1
  for (int run = k.run0; run * 16 < E; run += k.run_step) {
    float s1[NK * 4], w[KI];
#pragma unroll
    for (int i = 0; i < NK * 4; ++i) s1[i] = s0[i];
#pragma unroll
    for (int i = 0; i < KI; ++i) w[i] = v[i];
    load(run + k.run_step);
    const int e = run * 16 + l16;
#pragma unroll
    for (int ti = 0; ti < 4; ++ti) {
      if (ti * 16 >= count) break;
      ssd_floatx4 acc = {0.f, 0.f, 0.f, 0.f};
      const float* qr = Q + (ti * 16 + l16) * ks + grp * 4;
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const float4 qv = *reinterpret_cast<const float4*>(qr + i * 16);
        acc = ssd_mfma(qv.x, s1[i * 4 + 0], acc);
        acc = ssd_mfma(qv.y, s1[i * 4 + 1], acc);
        acc = ssd_mfma(qv.z, s1[i * 4 + 2], acc);
        acc = ssd_mfma(qv.w, s1[i * 4 + 3], acc);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[r] *= eL[ti][r];
#pragma unroll
      for (int tj = 0; tj <= ti; ++tj)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc = ssd_mfma(pf[ti * (ti + 1) / 2 + tj][c], w[tj * 4 + c], acc);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = ti * 16 + grp * 4 + r;  // the value of token t and column e is the fragment element the lane holds
        if (t < count && e < E) a.out[(size_t)(first + t) * ((size_t)a.H * E) + (size_t)h * E + e] = acc[r] + skip * w[ti * 4 + r];
      }
    }
  }
}

extern "C" int ms_ssd_chunk_tokens() { return SSD_CHUNK; }
extern "C" int ms_ssd_max_dim() { return SSD_MAX_DIM; }

// As ms_gated_recurrence in the step mode, in chunks. `chunks` = sum over the rows of ceil(tokens / SSD_CHUNK) (the host knows
// the rows' lengths); U [chunks, H, D E] and total [chunks, H] are scratch.
extern "C" int ms_ssd_chunked(const float* x, int ld, int q_off, int k_off, int v_off, int H, int D, int E, int share, const float* step,
                              int ld_step, const float* step_bias, const float* decay, const float* skip, float* S,
                              const int* row_start, const int* starts, const int* state_slots, float* out, int rows, int chunks,
                              float* U, float* total, hipStream_t st) {
  if (rows <= 0 || chunks <= 0) return MS_OK;
  if (H <= 0 || D <= 0 || E <= 0 || share < 1 || H % share || x == nullptr || step == nullptr || decay == nullptr || skip == nullptr ||
      S == nullptr || out == nullptr || row_start == nullptr || starts == nullptr || state_slots == nullptr || U == nullptr ||
      total == nullptr || q_off < 0 || k_off < 0 || v_off < 0 || q_off + H / share * D > ld || k_off + H / share * D > ld ||
      v_off + H * E > ld || ld_step < H)
    return MS_BAD_ARG;
  if (D > SSD_MAX_DIM || E > SSD_MAX_DIM || H > 65535 || rows > 65535) return MS_UNSUPPORTED;
  const int vec = D % 4 == 0 && E % 4 == 0 && ld % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0 && v_off % 4 == 0 && (size_t)x % 16 == 0;
  SsdArgs a{x, ld, q_off, k_off, v_off, H, D, E, share, step, ld_step, step_bias, decay, skip, S, row_start, starts, state_slots,
            out, U, total, rows, vec, share >= 4 ? 4 : share >= 2 ? 2 : 1};
  const int DP = (D + 15) & ~15;
  const int nk = DP <= 32 ? 2 : DP <= 64 ? 4 : DP <= 128 ? 8 : 16;
  const size_t lds1 = sizeof(float) * SSD_CHUNK * (size_t)(DP + 4);
  const int k_row = nk * 16 + 4, g_row = SSD_CHUNK + 4;
  const size_t lds3 = sizeof(float) * SSD_CHUNK * (size_t)(k_row + (k_row > g_row ? k_row : g_row));
  const void* out_kernel = nk == 2 ? (const void*)ssd_output_kernel<2> : nk == 4 ? (const void*)ssd_output_kernel<4>
                         : nk == 8 ? (const void*)ssd_output_kernel<8> : (const void*)ssd_output_kernel<16>;
  if (hipFuncSetAttribute((const void*)ssd_summary_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds1) != hipSuccess ||
      hipFuncSetAttribute(out_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds3) != hipSuccess)
    return MS_LAUNCH_FAILED;
  const dim3 per_chunk(chunks, H / share * ((share + a.HB - 1) / a.HB));
  ssd_summary_kernel<<<per_chunk, 256, lds1, st>>>(a);
  ssd_scan_kernel<<<dim3((D * E + 255) / 256, H, rows), 256, 0, st>>>(a);
  if (nk == 2) ssd_output_kernel<2><<<per_chunk, 256, lds3, st>>>(a);
  else if (nk == 4) ssd_output_kernel<4><<<per_chunk, 256, lds3, st>>>(a);
  else if (nk == 8) ssd_output_kernel<8><<<per_chunk, 256, lds3, st>>>(a);
  else ssd_output_kernel<16><<<per_chunk, 256, lds3, st>>>(a);
  return launch_status();
}
