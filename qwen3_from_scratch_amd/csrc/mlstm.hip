// The matrix memory of mLSTM: per head a matrix S (d x dv), a vector n (d) and a running maximum m,
//
//   i = cap tanh((z_i + b_i) / cap),   f = logsigmoid(cap tanh((z_f + b_f) / cap)),   m' = max(f + m, i),
//   S <- exp(f + m - m') S + exp(i - m') k v^T,   n <- exp(f + m - m') n + exp(i - m') k,
//   o = S^T q / (max(|n . q|, exp(-m')) + small),
//
// then o divided by its root mean square over the head, times a weight and sigmoid of a gate. A step's
// tokens are packed on one axis; sequence b owns rows cu[b] .. cu[b + 1] - 1 and the state at row
// slots[b] of the state tensor. A row of the input is float32 [q: H d | k: H d | v: H dv | gate: H dv |
// z_i: H | z_f: H], rows `row_stride` apart; q is multiplied by `q_scale` here. Everything is float32;
// sums of logarithms are double, since what counts is a small difference of two of them.
//
// The state of a request: S (H, d, dv), then n (H, tiles, d) and m (H, tiles) with tiles = dv / 64 rounded
// up: every 64 columns of a head have copies of n and m of their own (always equal), so that the
// workgroups of a decoding step need nothing from each other.
#include "common.h"

#define Q3_CHUNK 64
typedef __attribute__((ext_vector_type(4))) float mat4_t;

__device__ inline int mlstm_chunks_before(const int* __restrict__ cu, int b) {
  int n = 0;
  for (int i = 0; i < b; ++i) n += (cu[i + 1] - cu[i] + Q3_CHUNK - 1) / Q3_CHUNK;
  return n;
}

__device__ inline float capped_gate(float z, float cap) { return cap * tanhf(z / cap); }
__device__ inline float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ inline float gate_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }

struct MlstmShape {
  int H, d, dv, tiles;
  long row_stride, state_stride;
  float cap, q_scale, small, eps;
  __device__ const float* q(const float* rows, size_t t, int h) const { return rows + t * row_stride + (size_t)h * d; }
  __device__ const float* k(const float* rows, size_t t, int h) const { return rows + t * row_stride + (size_t)(H + h) * d; }
  __device__ const float* v(const float* rows, size_t t, int h) const {
    return rows + t * row_stride + 2 * (size_t)H * d + (size_t)h * dv;
  }
  __device__ const float* gate(const float* rows, size_t t, int h) const {
    return rows + t * row_stride + 2 * (size_t)H * d + (size_t)(H + h) * dv;
  }
  __device__ float z_i(const float* rows, size_t t, int h) const {
    return rows[t * row_stride + 2 * (size_t)H * (d + dv) + h];
  }
  __device__ float z_f(const float* rows, size_t t, int h) const {
    return rows[t * row_stride + 2 * (size_t)H * (d + dv) + H + h];
  }
  __device__ float* S(float* state, int h) const { return state + (size_t)h * d * dv; }
  __device__ float* n(float* state, int h, int tile) const {
    return state + (size_t)H * d * dv + ((size_t)h * tiles + tile) * d;
  }
  __device__ float* m(float* state, int h, int tile) const {
    return state + (size_t)H * d * dv + (size_t)H * tiles * d + (size_t)h * tiles + tile;
  }
};

// ---- steps of few rows ----
// grid (H * tiles, B), 256 threads: a block owns 64 columns of a head, a lane a column, a wavefront a
// quarter of the rows, whose numbers stay in registers over the sequence's tokens. The quarters' sums
// meet in shared memory. o is left as float32 in `raw` (T, H dv), undivided by its root mean square.
template <int RMAX>
__global__ void __launch_bounds__(256) mlstm_step_kernel(const float* __restrict__ rows, MlstmShape sh,
                                                         const float* __restrict__ i_bias, const float* __restrict__ f_bias,
                                                         float* __restrict__ state, const int* __restrict__ slots,
                                                         const int* __restrict__ cu, float* __restrict__ raw) {
  constexpr int NU = (RMAX + 63) / 64;       // rows of n a lane keeps
  __shared__ float sq[4 * RMAX], sk[4 * RMAX], part[4][64], part_n[4];
  const int h = blockIdx.x / sh.tiles, tile = blockIdx.x % sh.tiles, b = blockIdx.y;
  const int start = cu[b], end = cu[b + 1];
  if (end <= start) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int d = sh.d, dv = sh.dv;
  const int R = (d + 3) / 4, i0 = wave * R, rows_here = min(R, d - i0);     // this wavefront's rows of S
  const int j = tile * 64 + lane;
  const bool live = j < dv;
  float* mine = state + (size_t)slots[b] * sh.state_stride;
  float* Sp = sh.S(mine, h) + (size_t)i0 * dv + j;
  float S[RMAX], n[NU];
#pragma unroll
  for (int r = 0; r < RMAX; ++r) S[r] = (live && r < rows_here) ? Sp[(size_t)r * dv] : 0.f;
  float* np = sh.n(mine, h, tile) + i0;
#pragma unroll
  for (int u = 0; u < NU; ++u) n[u] = lane + 64 * u < rows_here ? np[lane + 64 * u] : 0.f;
  float m = *sh.m(mine, h, tile);
  for (int t = start; t < end; ++t) {
    __syncthreads();
    const float *q = sh.q(rows, t, h), *k = sh.k(rows, t, h);
    for (int i = threadIdx.x; i < d; i += 256) {
      // row i of S is row i % R of wavefront i / R
      sq[(i / R) * RMAX + i % R] = q[i] * sh.q_scale;
      sk[(i / R) * RMAX + i % R] = k[i];
    }
    const float gi = capped_gate(sh.z_i(rows, t, h) + i_bias[h], sh.cap);
    const float gf = log_sigmoid(capped_gate(sh.z_f(rows, t, h) + f_bias[h], sh.cap));
    const double kept = (double)gf + (double)m;
    const float m_new = (float)fmax(kept, (double)gi);
    const float keep = expf((float)(kept - (double)m_new)), enter = expf(gi - m_new);
    m = m_new;
    const float v = live ? sh.v(rows, t, h)[j] * enter : 0.f;
    __syncthreads();
    const float *wq = sq + wave * RMAX, *wk = sk + wave * RMAX;
    float acc = 0.f, dot = 0.f;
#pragma unroll
    for (int r = 0; r < RMAX; ++r) {
      if (r < rows_here) {
        S[r] = keep * S[r] + wk[r] * v;
        acc += S[r] * wq[r];
      }
    }
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      const int r = lane + 64 * u;
      if (r < rows_here) {
        n[u] = keep * n[u] + enter * wk[r];
        dot += n[u] * wq[r];
      }
    }
    dot = wave_sum(dot);
    part[wave][lane] = acc;
    if (lane == 0) part_n[wave] = dot;
    __syncthreads();
    if (wave == 0 && live) {
      const float num = (part[0][lane] + part[1][lane]) + (part[2][lane] + part[3][lane]);
      const float den = (part_n[0] + part_n[1]) + (part_n[2] + part_n[3]);
      raw[((size_t)t * sh.H + h) * dv + j] = num / (fmaxf(fabsf(den), expf(-m)) + sh.small);
    }
  }
#pragma unroll
  for (int r = 0; r < RMAX; ++r)
    if (live && r < rows_here) Sp[(size_t)r * dv] = S[r];
#pragma unroll
  for (int u = 0; u < NU; ++u)
    if (lane + 64 * u < rows_here) np[lane + 64 * u] = n[u];
  if (threadIdx.x == 0) *sh.m(mine, h, tile) = m;
}

// One wavefront per (token, head): o over its root mean square, times `norm` and sigmoid(gate).
template <typename TA>
__global__ void __launch_bounds__(64) mlstm_finish_kernel(const float* __restrict__ raw, const float* __restrict__ rows,
                                                          MlstmShape sh, const float* __restrict__ norm,
                                                          TA* __restrict__ out) {
  const int t = blockIdx.x, h = blockIdx.y;
  const float* o = raw + ((size_t)t * sh.H + h) * sh.dv;
  const float* gate = sh.gate(rows, t, h);
  float sq = 0.f;
  for (int j = threadIdx.x; j < sh.dv; j += 64) sq += o[j] * o[j];
  const float inv = rsqrtf(wave_sum(sq) / (float)sh.dv + sh.eps);
  for (int j = threadIdx.x; j < sh.dv; j += 64)
    out[((size_t)t * sh.H + h) * sh.dv + j] = from_float<TA>(o[j] * inv * norm[h * sh.dv + j] * gate_sigmoid(gate[j]));
}

// ---- many rows: chunks of 64 ----
// With b_t the sum of f over the chunk's rows up to and including t, a_s = i_s - b_s, and m0, S0, n0 the
// state before the chunk, let g_t = max(m0, max_{s <= t} a_s). Then m_t = b_t + g_t and
//
//   S_t = exp(m0 - g_t) S0 + sum_{s <= t} exp(a_s - g_t) k_s v_s^T,
//
// n_t likewise, every exponent at most zero. With A = max_s a_s over the chunk, the chunk's own sum
// U = sum_s exp(a_s - A) k_s v_s^T needs no m0. Four kernels: the gates and their sums; every chunk's own
// sum (all chunks at once); the states before every chunk, one chunk after the other; every chunk's results
// (all chunks at once). Products are float32 on the matrix cores (v_mfma_f32_16x16x4_f32: operand lane
// (r = lane % 16, k = lane / 16), result lane (column lane % 16, rows 4 (lane / 16) + 0 .. 3)).

// grid (chunks of the longest sequence, H / 4 rounded up, B): a wavefront per (chunk, head), a lane per row.
// Leaves b, a and the running maximum of a, double, (T, H) each.
__global__ void __launch_bounds__(256) mlstm_gates_kernel(const float* __restrict__ rows, MlstmShape sh,
                                                          const float* __restrict__ i_bias,
                                                          const float* __restrict__ f_bias, const int* __restrict__ cu,
                                                          double* __restrict__ sum_f, double* __restrict__ lift,
                                                          double* __restrict__ top) {
  const int b = blockIdx.z, c = blockIdx.x, h = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int start = cu[b], len = min(cu[b + 1] - start - c * Q3_CHUNK, Q3_CHUNK);
  if (len <= 0 || h >= sh.H) return;
  const size_t t = (size_t)start + c * Q3_CHUNK + lane;
  float gi = 0.f, gf = 0.f;
  if (lane < len) {
    gi = capped_gate(sh.z_i(rows, t, h) + i_bias[h], sh.cap);
    gf = log_sigmoid(capped_gate(sh.z_f(rows, t, h) + f_bias[h], sh.cap));
  }
  double run = (double)gf;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const double below = __shfl_up(run, off, 64);
    if (lane >= off) run += below;
  }
  const double a = (double)gi - run;
  double most = a;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const double below = __shfl_up(most, off, 64);
    if (lane >= off) most = fmax(most, below);
  }
  if (lane < len) {
    sum_f[t * sh.H + h] = run;
    lift[t * sh.H + h] = a;
    top[t * sh.H + h] = most;
  }
}

#define ML_LDA 68      // floats between rows of an operand whose 16 rows and 4 columns a read touches
#define ML_LDB 80      // ... whose 4 rows and 16 columns it touches

// grid (chunks of the longest sequence, H * tiles of 64 rows of S * tiles of 64 columns, B), 256 threads: 64 x 64
// numbers of the chunk's own sum U into `sums` (chunk, H, d dv + d), a wavefront 16 of the rows; the
// blocks of the first columns also form the sum of k alone, behind U.
__global__ void __launch_bounds__(256) mlstm_chunk_sums_kernel(const float* __restrict__ rows, MlstmShape sh,
                                                               const int* __restrict__ cu,
                                                               const double* __restrict__ lift,
                                                               const double* __restrict__ top, float* __restrict__ sums) {
  __shared__ __attribute__((aligned(16))) float kw[Q3_CHUNK * ML_LDB];
  __shared__ __attribute__((aligned(16))) float vt[Q3_CHUNK * ML_LDB];
  __shared__ float weight[Q3_CHUNK];
  const int b = blockIdx.z, c = blockIdx.x;
  const int start = cu[b], len = min(cu[b + 1] - start - c * Q3_CHUNK, Q3_CHUNK);
  if (len <= 0) return;
  const int d_tiles = (sh.d + 63) / 64;
  const int h = blockIdx.y / (sh.tiles * d_tiles), rest = blockIdx.y % (sh.tiles * d_tiles);
  const int tile = rest / d_tiles, i0 = rest % d_tiles * 64, j0 = tile * 64;
  const size_t row0 = (size_t)start + c * Q3_CHUNK;
  const size_t chunk = (size_t)mlstm_chunks_before(cu, b) + c;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15,
            grp = lane >> 4;
  // rows past the chunk's end have weight zero and are read from the last that exists, as are columns past the
  // head's, whose results nobody keeps: no load waits behind a branch
  const float *k0 = sh.k(rows, row0, h), *v0 = sh.v(rows, row0, h);
  const int stride = (int)sh.row_stride, k_col = min(i0 + lane, sh.d - 1), v_col = min(j0 + lane, sh.dv - 1);
  float gk[16], gv[16];
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int s = min(wave + 4 * u, len - 1) * stride;
    gk[u] = (k0 + s)[k_col];
    gv[u] = (v0 + s)[v_col];
  }
  if (tid < Q3_CHUNK)
    weight[tid] = tid < len ? expf((float)(lift[(row0 + tid) * sh.H + h] - top[(row0 + len - 1) * sh.H + h])) : 0.f;
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 16; ++u) {
    const int s = wave + 4 * u;
    kw[s * ML_LDB + lane] = gk[u] * weight[s];
    vt[s * ML_LDB + lane] = gv[u];
  }
  __syncthreads();
  mat4_t acc[4];
#pragma unroll
  for (int x = 0; x < 4; ++x) acc[x] = mat4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int s = 0; s < Q3_CHUNK; s += 4) {
    const float a = kw[(s + grp) * ML_LDB + 16 * wave + col];
#pragma unroll
    for (int x = 0; x < 4; ++x)
      acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, vt[(s + grp) * ML_LDB + 16 * x + col], acc[x], 0, 0, 0);
  }
  const size_t size = (size_t)sh.d * sh.dv + sh.d;
  float* dst = sums + (chunk * sh.H + h) * size;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int i = i0 + 16 * wave + 4 * grp + r;
    if (i < sh.d) {
#pragma unroll
      for (int x = 0; x < 4; ++x)
        if (j0 + 16 * x + col < sh.dv) dst[(size_t)i * sh.dv + j0 + 16 * x + col] = acc[x][r];
    }
  }
  if (tile == 0 && tid < 64 && i0 + tid < sh.d) {
    float n = 0.f;
    for (int s = 0; s < len; ++s) n += kw[s * ML_LDB + tid];
    dst[(size_t)sh.d * sh.dv + i0 + tid] = n;
  }
}

// grid ((d dv + d) / 256 rounded up, H, B): one number of S or n per thread, through the sequence's chunks in
// order. `sums` receives, in place of a chunk's own sum, the state before the chunk, and `before` (chunk, H) the
// m before it; the state tensor receives S and n after the last (m is the last results' to write: others here read it).
#define ML_AHEAD 8
__global__ void __launch_bounds__(256) mlstm_chunk_scan_kernel(float* __restrict__ sums, MlstmShape sh,
                                                               float* __restrict__ state, const int* __restrict__ slots,
                                                               const int* __restrict__ cu,
                                                               const double* __restrict__ sum_f,
                                                               const double* __restrict__ top, float* __restrict__ before) {
  const int h = blockIdx.y, b = blockIdx.z;
  const size_t size = (size_t)sh.d * sh.dv + sh.d, whole = (size_t)sh.d * sh.dv;
  const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x;
  const int start = cu[b], count = cu[b + 1] - start;
  if (count <= 0 || e >= size) return;
  const int chunks = (count + Q3_CHUNK - 1) / Q3_CHUNK;
  const size_t first = mlstm_chunks_before(cu, b);
  float* mine = state + (size_t)slots[b] * sh.state_stride;
  float X = e < whole ? sh.S(mine, h)[e] : sh.n(mine, h, 0)[e - whole];
  float m = *sh.m(mine, h, 0);
  for (int c0 = 0; c0 < chunks; c0 += ML_AHEAD) {
    float own[ML_AHEAD];
#pragma unroll
    for (int u = 0; u < ML_AHEAD; ++u)
      own[u] = c0 + u < chunks ? sums[((first + c0 + u) * sh.H + h) * size + e] : 0.f;
#pragma unroll
    for (int u = 0; u < ML_AHEAD; ++u) {
      if (c0 + u >= chunks) break;
      const size_t at = (first + c0 + u) * sh.H + h;
      const size_t last = (size_t)start + min((c0 + u + 1) * Q3_CHUNK, count) - 1;
      const double B = sum_f[last * sh.H + h], A = top[last * sh.H + h];
      sums[at * size + e] = X;
      if (e == 0) before[at] = m;
      // relative to the m that is kept, a float32 number, not to the double one
      const double kept = (double)m + B, come = A + B;
      const float m_new = (float)fmax(kept, come);
      X = expf((float)(kept - (double)m_new)) * X + expf((float)(come - (double)m_new)) * own[u];
      m = m_new;
    }
  }
  if (e < whole) {
    sh.S(mine, h)[e] = X;
  } else {
    for (int tile = 0; tile < sh.tiles; ++tile) sh.n(mine, h, tile)[e - whole] = X;
  }
}

// grid (chunks of the longest sequence, H * tiles, B), 256 threads: the chunk's results in 64 columns of one
// head, a wavefront 16 of its rows. First the weights W[t][s] = (q_t . k_s) exp(a_s - g_t), s <= t, into shared
// memory, and the denominators from their sums and q . n0; then exp(m0 - g_t) q S0 + W v over the denominator.
// A slice of 64 of the inner size is asked for while the one before it is worked on. With one tile a head's row
// is whole here and leaves over its root mean square, times `norm` and sigmoid(gate), into `out`; with more it
// goes to `raw` (T, H dv), and mlstm_finish_kernel follows.
template <typename TA, bool FINISH>
__global__ void __launch_bounds__(256) mlstm_chunk_output_kernel(
    const float* __restrict__ rows, MlstmShape sh, float* __restrict__ state, const int* __restrict__ slots,
    const int* __restrict__ cu, const double* __restrict__ sum_f, const double* __restrict__ lift,
    const double* __restrict__ top, const float* __restrict__ sums, const float* __restrict__ before,
    const float* __restrict__ norm, float* __restrict__ raw, TA* __restrict__ out) {
  __shared__ __attribute__((aligned(16))) float W[Q3_CHUNK * ML_LDA];
  __shared__ __attribute__((aligned(16))) float qs[Q3_CHUNK * ML_LDA];
  __shared__ __attribute__((aligned(16))) float other[Q3_CHUNK * ML_LDB];
  __shared__ float ns[64];
  __shared__ double lifts[Q3_CHUNK];
  const int b = blockIdx.z, h = blockIdx.y / sh.tiles, tile = blockIdx.y % sh.tiles, c = blockIdx.x;
  const int start = cu[b], count = cu[b + 1] - start, len = min(count - c * Q3_CHUNK, Q3_CHUNK);
  if (len <= 0) return;
  const int d = sh.d, dv = sh.dv, j0 = 64 * tile;
  const size_t row0 = (size_t)start + c * Q3_CHUNK;
  const size_t at = ((size_t)mlstm_chunks_before(cu, b) + c) * sh.H + h;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), col = lane & 15,
            grp = lane >> 4;
  const float* S0 = sums + at * ((size_t)d * dv + d);
  const float* n0 = S0 + (size_t)d * dv;
  const double m0 = (double)before[at];
  if (tid < Q3_CHUNK) lifts[tid] = tid < len ? lift[(row0 + tid) * sh.H + h] : 0.0;

  // What a thread brings of a slice: number `lane` of rows wave + 4 u: q (scaled) and k from column e0 on, S0
  // from row e0 on, v. Nothing branches: rows past the chunk's end and columns past the head's are read from
  // the last one that exists. Such rows of q make results that nobody keeps, such rows of k and v have weight
  // zero, and columns of q and k past the head's count as zero.
  float ga[16], gb[16];
  const float *q0 = sh.q(rows, row0, h), *k0 = sh.k(rows, row0, h), *v0 = sh.v(rows, row0, h);
  const int stride = (int)sh.row_stride, v_col = min(j0 + lane, dv - 1);
  auto ask_q = [&](int e0) {
    const int e = min(e0 + lane, d - 1);
#pragma unroll
    for (int u = 0; u < 16; ++u) ga[u] = (q0 + min(wave + 4 * u, len - 1) * stride)[e];
  };
  auto ask_k = [&](int e0) {
    const int e = min(e0 + lane, d - 1);
#pragma unroll
    for (int u = 0; u < 16; ++u) gb[u] = (k0 + min(wave + 4 * u, len - 1) * stride)[e];
  };
  auto ask_S = [&](int e0) {
#pragma unroll
    for (int u = 0; u < 16; ++u) gb[u] = (S0 + (size_t)min(e0 + wave + 4 * u, d - 1) * dv)[v_col];
  };
  auto ask_v = [&]() {
#pragma unroll
    for (int u = 0; u < 16; ++u) gb[u] = (v0 + min(wave + 4 * u, len - 1) * stride)[v_col];
  };
  auto put = [&](float (&from)[16], float* to, int apart, float scale) {
#pragma unroll
    for (int u = 0; u < 16; ++u) to[(wave + 4 * u) * apart + lane] = scale == 0.f ? 0.f : from[u] * scale;
  };

  mat4_t acc[4];
#pragma unroll
  for (int x = 0; x < 4; ++x) acc[x] = mat4_t{0.f, 0.f, 0.f, 0.f};
  float dot_n = 0.f;                    // row 16 wave + col's q . n0, the numbers 4 i + grp of it
  ask_q(0);
  ask_k(0);
  for (int e0 = 0; e0 < d; e0 += 64) {
    __syncthreads();
    put(ga, qs, ML_LDA, e0 + lane < d ? sh.q_scale : 0.f);
    put(gb, other, ML_LDA, e0 + lane < d ? 1.f : 0.f);
    if (tid < 64) ns[tid] = e0 + tid < d ? n0[e0 + tid] : 0.f;
    __syncthreads();
    if (e0 + 64 < d) {
      ask_q(e0 + 64);
      ask_k(e0 + 64);
    } else {
      if (d > 64) ask_q(0);             // the first slice of the product with S0; a single slice is still in place
      ask_S(0);
    }
#pragma unroll
    for (int i = 0; i < 64; i += 4) {
      const float a = qs[(16 * wave + col) * ML_LDA + i + grp];
      dot_n += a * ns[i + grp];
#pragma unroll
      for (int x = 0; x < 4; ++x)
        if (x <= wave)        // keys behind all of the wavefront's rows do not count
          acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, other[(16 * x + col) * ML_LDA + i + grp], acc[x], 0, 0, 0);
    }
  }
  dot_n += __shfl_xor(dot_n, 16, 64);
  dot_n += __shfl_xor(dot_n, 32, 64);
  float carry[4], under[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = 16 * wave + 4 * grp + r;
    const bool real = t < len;
    const double g = real ? fmax(m0, top[(row0 + t) * sh.H + h]) : 0.0;
    const double b_t = real ? sum_f[(row0 + t) * sh.H + h] : 0.0;
    float sum = 0.f;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int s = 16 * x + col;
      const float w = (real && s <= t) ? acc[x][r] * expf((float)(lifts[s] - g)) : 0.f;
      W[t * ML_LDA + s] = w;
      sum += w;
    }
#pragma unroll
    for (int off = 1; off < 16; off <<= 1) sum += __shfl_xor(sum, off, 64);
    carry[r] = real ? expf((float)(m0 - g)) : 0.f;
    const float den = sum + carry[r] * __shfl(dot_n, 4 * grp + r, 64);
    under[r] = 1.f / (fmaxf(fabsf(den), real ? expf((float)(-(b_t + g))) : 1.f) + sh.small);
  }
#pragma unroll
  for (int x = 0; x < 4; ++x) acc[x] = mat4_t{0.f, 0.f, 0.f, 0.f};
  for (int e0 = 0; e0 < d; e0 += 64) {
    __syncthreads();
    if (d > 64) put(ga, qs, ML_LDA, e0 + lane < d ? sh.q_scale : 0.f);
    put(gb, other, ML_LDB, 1.f);
    __syncthreads();
    if (e0 + 64 < d) {
      ask_q(e0 + 64);
      ask_S(e0 + 64);
    } else {
      ask_v();
    }
#pragma unroll
    for (int i = 0; i < 64; i += 4) {
      const float a = qs[(16 * wave + col) * ML_LDA + i + grp];
#pragma unroll
      for (int x = 0; x < 4; ++x)
        acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, other[(i + grp) * ML_LDB + 16 * x + col], acc[x], 0, 0, 0);
    }
  }
#pragma unroll
  for (int x = 0; x < 4; ++x)
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[x][r] *= carry[r];
  __syncthreads();
  put(gb, other, ML_LDB, 1.f);
  __syncthreads();
  for (int s = 0; s < 16 * (wave + 1); s += 4) {
    const float a = W[(16 * wave + col) * ML_LDA + s + grp];
#pragma unroll
    for (int x = 0; x < 4; ++x)
      acc[x] = __builtin_amdgcn_mfma_f32_16x16x4f32(a, other[(s + grp) * ML_LDB + 16 * x + col], acc[x], 0, 0, 0);
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int t = 16 * wave + 4 * grp + r;
    const float* gate = sh.gate(rows, row0 + (t < len ? t : 0), h);
    float inv = 1.f;
    if (FINISH) {
      float sq = 0.f;
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float o = 16 * x + col < dv ? acc[x][r] * under[r] : 0.f;
        sq += o * o;
      }
#pragma unroll
      for (int off = 1; off < 16; off <<= 1) sq += __shfl_xor(sq, off, 64);
      inv = rsqrtf(sq / (float)dv + sh.eps);
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int j = j0 + 16 * x + col;
      if (t < len && j < dv) {
        const size_t place = ((row0 + t) * sh.H + h) * dv + j;
        const float o = acc[x][r] * under[r];
        if (FINISH)
          out[place] = from_float<TA>(o * inv * norm[h * dv + j] * gate_sigmoid(gate[j]));
        else
          raw[place] = o;
      }
    }
  }
  // the m after the sequence's last row: as the scan has it
  if ((c + 1) * Q3_CHUNK >= count && tid == 0) {
    const size_t last = row0 + len - 1;
    const double B = sum_f[last * sh.H + h];
    *sh.m(state + (size_t)slots[b] * sh.state_stride, h, tile) = (float)fmax(m0 + B, top[last * sh.H + h] + B);
  }
}

static bool mlstm_shape(MlstmShape& sh, int H, int d, int dv, long row_stride, long state_stride, float cap, float small,
                        float eps) {
  if (H <= 0 || d <= 0 || dv <= 0 || !(cap > 0.f) || row_stride < 2L * H * (d + dv) + 2L * H) return false;
  sh.H = H, sh.d = d, sh.dv = dv, sh.tiles = (dv + 63) / 64;
  if (state_stride < (long)H * d * dv + (long)H * sh.tiles * (d + 1)) return false;
  sh.row_stride = row_stride, sh.state_stride = state_stride;
  sh.cap = cap, sh.q_scale = (float)(1.0 / sqrt((double)d)), sh.small = small, sh.eps = eps;
  return true;
}

// Numbers of a request's state, and bytes of workspace for a step of T rows in B sequences (`chunked` or not).
extern "C" long q3_mlstm_state_numbers(int H, int d, int dv) {
  return (long)H * d * dv + (long)H * ((dv + 63) / 64) * (d + 1);
}

extern "C" long q3_mlstm_workspace(int T, int B, int H, int d, int dv, int chunked) {
  const long raw = (long)T * H * dv * 4;
  if (!chunked) return raw;
  const long chunks = T / Q3_CHUNK + B;
  return 3L * T * H * 8 + chunks * H * ((long)d * dv + d) * 4 + chunks * H * 4 + raw;
}

extern "C" int q3_mlstm_scan(const float* rows, long row_stride, const float* i_bias, const float* f_bias, float cap,
                             const float* norm, float eps, float small, float* state, long state_stride, const int* slots,
                             const int* cu, void* out, void* workspace, int T, int B, int max_q_len, int H, int d, int dv,
                             int chunked, int act_dtype, hipStream_t stream) {
  MlstmShape sh;
  if (T <= 0 || B <= 0 || max_q_len <= 0 || !mlstm_shape(sh, H, d, dv, row_stride, state_stride, cap, small, eps))
    return Q3_ERR_BAD_ARGUMENT;
  const long d_tiles = (d + 63) / 64;
  if (d > 512 || row_stride > (1 << 24) || B > 65535 || (long)H * sh.tiles * d_tiles > 65535 || sh.tiles > 256) return Q3_ERR_UNSUPPORTED;
  if (!chunked) {
    float* raw = (float*)workspace;
    const dim3 grid(H * sh.tiles, B);
    const int R = (d + 3) / 4;
#define Q3_MLSTM_STEP(RM) \
  hipLaunchKernelGGL(mlstm_step_kernel<RM>, grid, dim3(256), 0, stream, rows, sh, i_bias, f_bias, state, slots, cu, raw)
    if (R <= 16)
      Q3_MLSTM_STEP(16);
    else if (R <= 32)
      Q3_MLSTM_STEP(32);
    else if (R <= 64)
      Q3_MLSTM_STEP(64);
    else
      Q3_MLSTM_STEP(128);
#undef Q3_MLSTM_STEP
    Q3_DISPATCH_DTYPE(act_dtype, TA,
                      hipLaunchKernelGGL(mlstm_finish_kernel<TA>, dim3(T, H), dim3(64), 0, stream, raw, rows, sh, norm,
                                         (TA*)out));
    return q3_launch_status();
  }
  const size_t chunks_all = (size_t)(T / Q3_CHUNK + B);
  double* sum_f = (double*)workspace;
  double* lift = sum_f + (size_t)T * H;
  double* top = lift + (size_t)T * H;
  float* sums = (float*)(top + (size_t)T * H);
  const size_t size = (size_t)d * dv + d;
  float* before = sums + chunks_all * H * size;
  float* raw = before + chunks_all * H;
  const int chunks = (max_q_len + Q3_CHUNK - 1) / Q3_CHUNK;
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3(chunks, (H + 3) / 4, B), dim3(256), 0, stream, rows, sh, i_bias, f_bias, cu,
                     sum_f, lift, top);
  hipLaunchKernelGGL(mlstm_chunk_sums_kernel, dim3(chunks, (int)(H * sh.tiles * d_tiles), B), dim3(256), 0, stream, rows, sh,
                     cu, lift, top, sums);
  hipLaunchKernelGGL(mlstm_chunk_scan_kernel, dim3((unsigned)((size + 255) / 256), H, B), dim3(256), 0, stream, sums, sh,
                     state, slots, cu, sum_f, top, before);
  if (sh.tiles == 1) {
    Q3_DISPATCH_DTYPE(act_dtype, TA,
                      hipLaunchKernelGGL((mlstm_chunk_output_kernel<TA, true>), dim3(chunks, H, B), dim3(256), 0, stream,
                                         rows, sh, state, slots, cu, sum_f, lift, top, sums, before, norm, raw, (TA*)out));
    return q3_launch_status();
  }
  hipLaunchKernelGGL((mlstm_chunk_output_kernel<float, false>), dim3(chunks, H * sh.tiles, B), dim3(256), 0, stream, rows,
                     sh, state, slots, cu, sum_f, lift, top, sums, before, norm, raw, (float*)nullptr);
  Q3_DISPATCH_DTYPE(act_dtype, TA,
                    hipLaunchKernelGGL(mlstm_finish_kernel<TA>, dim3(T, H), dim3(64), 0, stream, raw, rows, sh, norm,
                                       (TA*)out));
  return q3_launch_status();
}
