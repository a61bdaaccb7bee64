// Softmax attention with biased projections, a norm over the whole query and key projections,
// a rotation of neighbouring pairs, capped scores, key and value heads of different sizes and a
// gate per head, over a paged cache: keys (pages, G, page, dim), values (pages, G, page, vdim) or,
// transposed within the page as the matrix-core kernels read them, (pages, G, vdim, page).
#include "common.h"

// One block per token. The row is [q: H dim | k: G dim | v: G vdim | ...] float32, `bias` covers
// q, k and v (null: projections without biases). q and k (bias added) are each divided by the root mean square of the whole
// projection and multiplied by their weight, then the first 2 * half numbers of every head turn
// in pairs (2i, 2i + 1) by position * inv_freq[i]. q goes to `q_out`, k and v (bias added) into
// the token's place in the cache, when one is given.
template <typename TA>
__global__ void softcap_prepare_kernel(const float* __restrict__ rows, long row_stride, const float* __restrict__ bias,
                                       const float* __restrict__ q_weight, const float* __restrict__ k_weight, float eps,
                                       const float* __restrict__ inv_freq, int half, const int* __restrict__ positions,
                                       const int* __restrict__ seq_index, const int* __restrict__ block_table,
                                       int table_width, TA* __restrict__ k_cache, TA* __restrict__ v_cache, int page,
                                       TA* __restrict__ q_out, int H, int G, int dim, int vdim, int v_transposed) {
  __shared__ float scratch[17];
  const int t = blockIdx.x;
  const float* row = rows + (size_t)t * row_stride;
  const int nq = H * dim, nk = G * dim, nv = G * vdim;
  float sq = 0.f, sk = 0.f;
  for (int j = threadIdx.x; j < nq; j += blockDim.x) {
    const float z = row[j] + (bias ? bias[j] : 0.f);
    sq += z * z;
  }
  for (int j = threadIdx.x; j < nk; j += blockDim.x) {
    const float z = row[nq + j] + (bias ? bias[nq + j] : 0.f);
    sk += z * z;
  }
  const float rq = rsqrtf(block_sum(sq, scratch) / (float)nq + eps);
  const float rk = rsqrtf(block_sum(sk, scratch) / (float)nk + eps);
  const int pos = positions[t];
  const float fpos = (float)pos;
  for (int j = threadIdx.x; j < nq; j += blockDim.x) {
    const int e = j % dim;
    float own = (row[j] + (bias ? bias[j] : 0.f)) * rq * q_weight[j];
    if (e < 2 * half) {
      const int p = j ^ 1;
      const float other = (row[p] + (bias ? bias[p] : 0.f)) * rq * q_weight[p];
      const float angle = fpos * inv_freq[e >> 1];
      const float c = cosf(angle), s = sinf(angle);
      own = (e & 1) ? own * c + other * s : own * c - other * s;
    }
    q_out[(size_t)t * nq + j] = from_float<TA>(own);
  }
  if (!k_cache) return;
  const int pg = block_table[(size_t)seq_index[t] * table_width + pos / page];
  if (pg < 0) return;
  const int off = pos % page;
  for (int j = threadIdx.x; j < nk; j += blockDim.x) {
    const int g = j / dim, e = j % dim;
    float own = (row[nq + j] + (bias ? bias[nq + j] : 0.f)) * rk * k_weight[j];
    if (e < 2 * half) {
      const int p = j ^ 1;
      const float other = (row[nq + p] + (bias ? bias[nq + p] : 0.f)) * rk * k_weight[p];
      const float angle = fpos * inv_freq[e >> 1];
      const float c = cosf(angle), s = sinf(angle);
      own = (e & 1) ? own * c + other * s : own * c - other * s;
    }
    k_cache[(((size_t)pg * G + g) * page + off) * dim + e] = from_float<TA>(own);
  }
  for (int j = threadIdx.x; j < nv; j += blockDim.x) {
    const int g = j / vdim, e = j % vdim;
    const size_t at = v_transposed ? (((size_t)pg * G + g) * vdim + e) * page + off
                                   : (((size_t)pg * G + g) * page + off) * vdim + e;
    v_cache[at] = from_float<TA>(row[nq + nk + j] + (bias ? bias[nq + nk + j] : 0.f));
  }
}

// Queries, keys and values turned by the position, i and i + half together. grid (T,
// shares): a token's heads (queries', then keys') go over the wavefronts of its blocks in turn. The row is [q: H dim | k: G dim | v: G vdim | ...] float32,
// `bias` covers q, k and v (null: none); with `values_are_keys` there is no v and a token's value is
// its key before it turns. The first 2 * half numbers of every head of q and k turn by position *
// inv_freq[i], cos and sin multiplied by `factor`; they are formed once per token, in shared memory. q
// goes to `q_out`, k and v into the token's place in the cache.
//
// `norm.on`: a head of q or k is divided by its own root mean square and multiplied by `q_weight` or
// `k_weight` (dim numbers that the heads share; null: by nothing) before it turns. `mix.first`: a token's
// value is (1 - share) v + share first, first's rows [G vdim] a stride apart.
//
// `runs` (single tokens only): a token that ends a run of `pool` tokens also leaves the means of the
// run's keys and values, as the cache holds them, in the run's place: the others' are read from the
// cache, where earlier steps have put them, its own are at hand.
#define Q3_TURN_HALF_MOST 256
struct RunPlaces {
  void* k;               // (pages, G, page, dim)
  void* v;               // (pages, G, vdim, page)
  const int* table;
  int width, pool;
};
struct HeadNorm {
  int on;
  float eps;
  const float* q_weight;
  const float* k_weight;
};
struct ValueMix {
  const float* first;
  long stride;
  const float* share;
};

// The sum of one number of a head over tokens first .. last - 1, in their order, from a paged cache: token j's
// stands at element `offset + (j % page) * apart` of its page's head. Sixteen loads are asked for before the
// first is used, none behind a branch (past the end the last token's are read again and not counted).
template <typename TA>
__device__ inline float sum_over_tokens(const TA* cache, const int* __restrict__ table, int first, int last, int page, int G,
                                        int g, size_t head_size, size_t offset, int apart) {
  float sum = 0.f;
  for (int j0 = first; j0 < last; j0 += 16) {
    int pages[16];
    TA got[16];
#pragma unroll
    for (int u = 0; u < 16; ++u) pages[u] = table[min(j0 + u, last - 1) / page];
#pragma unroll
    for (int u = 0; u < 16; ++u) {
      const int slot = min(j0 + u, last - 1) % page;
      got[u] = cache[((size_t)max(pages[u], 0) * G + g) * head_size + offset + (size_t)slot * apart];
    }
#pragma unroll
    for (int u = 0; u < 16; ++u) sum += (j0 + u < last && pages[u] >= 0) ? to_float(got[u]) : 0.f;
  }
  return sum;
}

template <typename TA>
__global__ void __launch_bounds__(256) turn_prepare_kernel(
    const float* __restrict__ rows, long row_stride, const float* __restrict__ bias, const float* __restrict__ inv_freq,
    int half, float factor, const int* __restrict__ positions, const int* __restrict__ seq_index,
    const int* __restrict__ block_table, int table_width, TA* k_cache, TA* v_cache, int page, TA* __restrict__ q_out,
    int H, int G, int dim, int vdim, int values_are_keys, RunPlaces runs, HeadNorm norm, ValueMix mix) {
  __shared__ float cs[Q3_TURN_HALF_MOST], sn[Q3_TURN_HALF_MOST];
  const int t = blockIdx.x;
  const int lane = threadIdx.x % Q3_WAVE, waves = blockDim.x / Q3_WAVE * gridDim.y;
  const int wave = blockIdx.y * (blockDim.x / Q3_WAVE) + threadIdx.x / Q3_WAVE;
  const float* row = rows + (size_t)t * row_stride;
  const int nq = H * dim, nk = G * dim;
  const int pos = positions[t];
  for (int i = threadIdx.x; i < half; i += blockDim.x) {
    const float angle = (float)pos * inv_freq[i];
    cs[i] = cosf(angle) * factor;
    sn[i] = sinf(angle) * factor;
  }
  const int* table = block_table + (size_t)seq_index[t] * table_width;
  const int pg = pos / page < table_width ? table[pos / page] : -1;
  const int off = pos % page;
  const bool ends_run = runs.k && (pos + 1) % runs.pool == 0;
  int run_page = -1, run_off = 0;
  if (ends_run) {
    const int r = pos / runs.pool;
    if (r / page < runs.width) run_page = runs.table[(size_t)seq_index[t] * runs.width + r / page];
    run_off = r % page;
  }
  __syncthreads();
  // the factor of a head's numbers: one over its root mean square, in every lane
  auto head_scale = [&](const float* x, const float* add) {
    if (!norm.on) return 1.f;
    float acc = 0.f;
    for (int e = lane; e < dim; e += Q3_WAVE) {
      const float z = x[e] + (add ? add[e] : 0.f);
      acc += z * z;
    }
    return rsqrtf(wave_sum(acc) / (float)dim + norm.eps);
  };
  auto turned = [&](const float* x, const float* add, float scale, const float* weight, int e) {
    const float own = (x[e] + (add ? add[e] : 0.f)) * (weight ? scale * weight[e] : scale);
    if (e >= 2 * half) return own;
    const int p = e < half ? e + half : e - half;
    const float other = (x[p] + (add ? add[p] : 0.f)) * (weight ? scale * weight[p] : scale);
    return e < half ? own * cs[e] - other * sn[e] : own * cs[p] + other * sn[p];
  };
  for (int h = wave; h < H; h += waves) {
    const float* x = row + h * dim;
    const float* add = bias ? bias + h * dim : nullptr;
    const float scale = head_scale(x, add);
    for (int e = lane; e < dim; e += Q3_WAVE)
      q_out[(size_t)t * nq + h * dim + e] = from_float<TA>(turned(x, add, scale, norm.q_weight, e));
  }
  if (pg < 0) return;
  int g = wave - H % waves;                    // the wavefront after the last query head's takes the first key head
  for (g = g < 0 ? g + waves : g; g < G; g += waves) {
    const float* x = row + nq + g * dim;
    const float* add = bias ? bias + nq + g * dim : nullptr;
    const float scale = head_scale(x, add);
    for (int e = lane; e < dim; e += Q3_WAVE) {
      const TA key = from_float<TA>(turned(x, add, scale, norm.k_weight, e));
      k_cache[(((size_t)pg * G + g) * page + off) * dim + e] = key;
      if (run_page >= 0) {
        const float sum = sum_over_tokens<TA>(k_cache, table, pos - runs.pool + 1, pos, page, G, g, (size_t)page * dim, e, dim) +
                          to_float(key);
        ((TA*)runs.k)[(((size_t)run_page * G + g) * page + run_off) * dim + e] = from_float<TA>(sum / (float)runs.pool);
      }
    }
    const float* y = values_are_keys ? x : row + nq + nk + g * vdim;
    const float* add_v = values_are_keys ? add : (bias ? bias + nq + nk + g * vdim : nullptr);
    for (int e = lane; e < vdim; e += Q3_WAVE) {
      float own = y[e] + (add_v ? add_v[e] : 0.f);
      if (mix.first) own = (1.f - *mix.share) * own + *mix.share * mix.first[(size_t)t * mix.stride + g * vdim + e];
      const TA value = from_float<TA>(own);
      v_cache[(((size_t)pg * G + g) * vdim + e) * page + off] = value;
      if (run_page >= 0) {
        const float sum = sum_over_tokens<TA>(v_cache, table, pos - runs.pool + 1, pos, page, G, g, (size_t)page * vdim,
                                              (size_t)e * page, 1) +
                          to_float(value);
        ((TA*)runs.v)[(((size_t)run_page * G + g) * vdim + e) * page + run_off] = from_float<TA>(sum / (float)runs.pool);
      }
    }
  }
}

// The same for sizes in steps of four and no runs, in 16-byte accesses: LPH lanes to a head, so that a wavefront
// works on 64 / LPH heads (queries', then keys', then values') at once. A lane holds four numbers of the part
// that turns and the four they turn with, or four of what passes, or four of a value.
__device__ inline void put4(float* at, float4 v) { *reinterpret_cast<float4*>(at) = v; }
__device__ inline void put4(bf16_t* at, float4 v) {
  union {
    uint2 u;
    __bf16 e[4];
  } pk;
  pk.e[0] = (__bf16)v.x; pk.e[1] = (__bf16)v.y; pk.e[2] = (__bf16)v.z; pk.e[3] = (__bf16)v.w;
  *reinterpret_cast<uint2*>(at) = pk.u;
}
__device__ inline void put1(float* at, float v) { *at = v; }
__device__ inline void put1(bf16_t* at, float v) { *reinterpret_cast<__bf16*>(at) = (__bf16)v; }
__device__ inline float4 get4(const float* at) { return *reinterpret_cast<const float4*>(at); }
__device__ inline float4 plus4(float4 a, float4 b) { return make_float4(a.x + b.x, a.y + b.y, a.z + b.z, a.w + b.w); }
__device__ inline float4 times4(float4 a, float4 b) { return make_float4(a.x * b.x, a.y * b.y, a.z * b.z, a.w * b.w); }
__device__ inline float4 scaled4(float4 a, float f) { return make_float4(a.x * f, a.y * f, a.z * f, a.w * f); }
__device__ inline float squares4(float4 a) { return a.x * a.x + a.y * a.y + a.z * a.z + a.w * a.w; }

template <typename TA, int LPH>
__global__ void __launch_bounds__(256) turn_prepare_vec_kernel(
    const float* __restrict__ rows, long row_stride, const float* __restrict__ bias, const float* __restrict__ inv_freq,
    int half, float factor, const int* __restrict__ positions, const int* __restrict__ seq_index,
    const int* __restrict__ block_table, int table_width, TA* __restrict__ k_cache, TA* __restrict__ v_cache, int page,
    TA* __restrict__ q_out, int H, int G, int dim, int vdim, int values_are_keys, HeadNorm norm, ValueMix mix) {
  __shared__ __align__(16) float cs[Q3_TURN_HALF_MOST], sn[Q3_TURN_HALF_MOST];
  constexpr int PER = Q3_WAVE / LPH;
  const int t = blockIdx.x;
  const int lane = threadIdx.x % Q3_WAVE, l = lane % LPH;
  const int step = blockDim.x / Q3_WAVE * gridDim.y * PER;
  const int first_item = (blockIdx.y * (blockDim.x / Q3_WAVE) + threadIdx.x / Q3_WAVE) * PER + lane / LPH;
  const float* row = rows + (size_t)t * row_stride;
  const int heads = H + G, items = H + 2 * G, turning = half / 4, lanes = turning + (dim - 2 * half) / 4;
  const int pos = positions[t];
  for (int i = threadIdx.x; i < half; i += blockDim.x) {
    float s, c;
    sincosf((float)pos * inv_freq[i], &s, &c);
    cs[i] = c * factor;
    sn[i] = s * factor;
  }
  const int pg = pos / page < table_width ? block_table[(size_t)seq_index[t] * table_width + pos / page] : -1;
  const int off = pos % page;
  const float share = mix.first ? *mix.share : 0.f;
  const bool turns = l < turning, holds = l < lanes;
  const int at = turns ? 4 * l : 2 * half + 4 * (l - turning);    // where this lane's first four numbers stand in a head
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  __syncthreads();
  for (int item = first_item; item < items; item += step) {
    if (item < heads) {
      const float* x = row + (size_t)item * dim;
      float4 a = holds ? get4(x + at) : zero, b = turns ? get4(x + half + at) : zero;
      if (bias) {
        const float* add = bias + (size_t)item * dim;
        if (holds) a = plus4(a, get4(add + at));
        if (turns) b = plus4(b, get4(add + half + at));
      }
      if (norm.on) {
        float acc = squares4(a) + squares4(b);
#pragma unroll
        for (int o = LPH / 2; o > 0; o >>= 1) acc += __shfl_xor(acc, o, Q3_WAVE);
        const float scale = rsqrtf(acc / (float)dim + norm.eps);
        a = scaled4(a, scale);
        b = scaled4(b, scale);
        const float* weight = item < H ? norm.q_weight : norm.k_weight;
        if (weight) {
          if (holds) a = times4(a, get4(weight + at));
          if (turns) b = times4(b, get4(weight + half + at));
        }
      }
      TA* dst = item < H ? q_out + ((size_t)t * H + item) * dim
                         : k_cache + (((size_t)max(pg, 0) * G + item - H) * page + off) * dim;
      if (item >= H && pg < 0) continue;
      if (turns) {
        const float4 c = get4(cs + at), s = get4(sn + at);
        put4(dst + half + at, make_float4(b.x * c.x + a.x * s.x, b.y * c.y + a.y * s.y, b.z * c.z + a.z * s.z, b.w * c.w + a.w * s.w));
        a = make_float4(a.x * c.x - b.x * s.x, a.y * c.y - b.y * s.y, a.z * c.z - b.z * s.z, a.w * c.w - b.w * s.w);
      }
      if (holds) put4(dst + at, a);
    } else if (pg >= 0 && 4 * l < vdim) {
      const int g = item - heads;
      const size_t from = values_are_keys ? (size_t)(H + g) * dim : (size_t)heads * dim + (size_t)g * vdim;
      float4 v = get4(row + from + 4 * l);
      if (bias) v = plus4(v, get4(bias + from + 4 * l));
      if (mix.first)
        v = plus4(scaled4(v, 1.f - share), scaled4(get4(mix.first + (size_t)t * mix.stride + (size_t)g * vdim + 4 * l), share));
      TA* dst = v_cache + (((size_t)pg * G + g) * vdim + 4 * l) * page + off;
      put1(dst, v.x);
      put1(dst + page, v.y);
      put1(dst + 2 * (size_t)page, v.z);
      put1(dst + 3 * (size_t)page, v.w);
    }
  }
}

extern "C" int q3_turn_prepare(const float* rows, long row_stride, const float* bias, const float* inv_freq, int half,
                               float factor, const int* positions, const int* seq_index, const int* block_table,
                               int table_width, void* k_cache, void* v_cache, int page, void* q_out, int T, int H, int G,
                               int dim, int vdim, int values_are_keys, void* run_k, void* run_v, const int* run_table,
                               int run_width, int pool, int norm_on, float norm_eps, const float* q_weight,
                               const float* k_weight, const float* mix_first, long mix_stride, const float* mix_share,
                               int act_dtype, hipStream_t stream) {
  if (T <= 0 || H <= 0 || G <= 0 || H % G || dim <= 0 || vdim <= 0 || half < 0 || 2 * half > dim || !k_cache || !v_cache ||
      !block_table || page <= 0 || table_width <= 0 || (half > 0 && !inv_freq) || (values_are_keys && dim != vdim))
    return Q3_ERR_BAD_ARGUMENT;
  if (run_k && (!run_v || !run_table || run_width <= 0 || pool <= 0)) return Q3_ERR_BAD_ARGUMENT;
  if ((mix_first && (!mix_share || values_are_keys)) || (q_weight == nullptr) != (k_weight == nullptr) || (q_weight && !norm_on))
    return Q3_ERR_BAD_ARGUMENT;
  if (half > Q3_TURN_HALF_MOST) return Q3_ERR_UNSUPPORTED;
  const RunPlaces runs{run_k, run_v, run_table, run_width, pool};
  const HeadNorm norm{norm_on, norm_eps, q_weight, k_weight};
  const ValueMix mix{mix_first, mix_stride, mix_share};
  // few tokens: a wavefront per head; many: the tokens fill the chip, and share their cosines among more heads
  const auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
  int lanes = half / 4 + (dim - 2 * half) / 4;
  if (vdim / 4 > lanes) lanes = vdim / 4;
  if (!run_k && half % 4 == 0 && dim % 4 == 0 && vdim % 4 == 0 && lanes <= 64 && row_stride % 4 == 0 && mix_stride % 4 == 0 &&
      aligned(rows) && aligned(bias) && aligned(q_weight) && aligned(k_weight) && aligned(mix_first) && aligned(k_cache) &&
      aligned(q_out)) {
    const int lph = lanes <= 16 ? 16 : lanes <= 32 ? 32 : 64;
    const int waves = ((H + 2 * G) * lph + Q3_WAVE - 1) / Q3_WAVE, blocks = (waves + 3) / 4;
    const int shares = T >= 1024 ? 1 : (T >= 256 ? (blocks < 2 ? blocks : 2) : (blocks < 64 ? blocks : 64));
#define Q3_TURN_VEC(LPH)                                                                                                     \
  Q3_DISPATCH_DTYPE(act_dtype, TA,                                                                                         \
                    hipLaunchKernelGGL((turn_prepare_vec_kernel<TA, LPH>), dim3(T, shares), dim3(256), 0, stream, rows,      \
                                       row_stride, bias, inv_freq, half, factor, positions, seq_index, block_table,         \
                                       table_width, (TA*)k_cache, (TA*)v_cache, page, (TA*)q_out, H, G, dim, vdim,          \
                                       values_are_keys, norm, mix))
    if (lph == 16)
      Q3_TURN_VEC(16);
    else if (lph == 32)
      Q3_TURN_VEC(32);
    else
      Q3_TURN_VEC(64);
#undef Q3_TURN_VEC
    return q3_launch_status();
  }
  const int most = (H + G + 3) / 4;
  const int shares = T >= 1024 ? 1 : (T >= 256 ? (most < 2 ? most : 2) : (most < 64 ? most : 64));
  Q3_DISPATCH_DTYPE(act_dtype, TA,
                    hipLaunchKernelGGL(turn_prepare_kernel<TA>, dim3(T, shares), dim3(256), 0, stream, rows, row_stride, bias,
                                       inv_freq, half, factor, positions, seq_index, block_table, table_width,
                                       (TA*)k_cache, (TA*)v_cache, page, (TA*)q_out, H, G, dim, vdim, values_are_keys,
                                       runs, norm, mix));
  return q3_launch_status();
}

// The same means for steps of any rows, after the step's keys and values are in the cache: grid (runs
// that a sequence may complete, G, B), a block per run; a run is formed if the step brought its last
// token. Sums take the tokens in their order, as above.
template <typename TA>
__global__ void __launch_bounds__(256) pool_runs_kernel(const TA* __restrict__ k_cache, const TA* __restrict__ v_cache,
                                                        const int* __restrict__ block_table, int table_width,
                                                        const int* __restrict__ cu, const int* __restrict__ kv_lens,
                                                        TA* __restrict__ run_k, TA* __restrict__ run_v,
                                                        const int* __restrict__ run_table, int run_width, int pool, int G,
                                                        int dim, int vdim, int page) {
  const int b = blockIdx.z, g = blockIdx.y;
  const int kv_len = kv_lens[b], first_pos = kv_len - (cu[b + 1] - cu[b]);
  const int r = first_pos / pool + blockIdx.x;          // first_pos's own run is the first that may end now
  if (kv_len <= first_pos || (r + 1) * pool > kv_len || r / page >= run_width) return;
  const int run_page = run_table[(size_t)b * run_width + r / page];
  if (run_page < 0) return;
  const int run_off = r % page;
  const int* table = block_table + (size_t)b * table_width;
  for (int e = threadIdx.x; e < dim + vdim; e += blockDim.x) {
    const bool key = e < dim;
    const int c = key ? e : e - dim;
    const float sum = key ? sum_over_tokens<TA>(k_cache, table, r * pool, (r + 1) * pool, page, G, g, (size_t)page * dim, c, dim)
                          : sum_over_tokens<TA>(v_cache, table, r * pool, (r + 1) * pool, page, G, g, (size_t)page * vdim,
                                                (size_t)c * page, 1);
    const size_t head = (size_t)run_page * G + g;
    const TA mean = from_float<TA>(sum / (float)pool);
    if (key)
      run_k[(head * page + run_off) * dim + c] = mean;
    else
      run_v[(head * vdim + c) * page + run_off] = mean;
  }
}

extern "C" int q3_pool_runs(const void* k_cache, const void* v_cache, const int* block_table, int table_width,
                            const int* cu, const int* kv_lens, void* run_k, void* run_v, const int* run_table,
                            int run_width, int pool, int B, int max_q_len, int G, int dim, int vdim, int page,
                            int act_dtype, hipStream_t stream) {
  if (B <= 0 || max_q_len <= 0 || G <= 0 || dim <= 0 || vdim <= 0 || page <= 0 || pool <= 0 || table_width <= 0 ||
      run_width <= 0 || !k_cache || !v_cache || !run_k || !run_v || !block_table || !run_table)
    return Q3_ERR_BAD_ARGUMENT;
  if (B > 65535 || G > 65535) return Q3_ERR_UNSUPPORTED;
  // a step of n tokens ends at most (n + pool - 1) / pool runs
  const int most = (max_q_len + pool - 1) / pool;
  Q3_DISPATCH_DTYPE(act_dtype, TA,
                    hipLaunchKernelGGL(pool_runs_kernel<TA>, dim3(most, G, B), dim3(256), 0, stream, (const TA*)k_cache,
                                       (const TA*)v_cache, block_table, table_width, cu, kv_lens, (TA*)run_k, (TA*)run_v,
                                       run_table, run_width, pool, G, dim, vdim, page));
  return q3_launch_status();
}

// The general form: one wavefront per (token, head). Keys are taken in tiles of 64 that start at
// absolute positions in steps of 64, one key a lane: score = (q . k) scale, capped as
// cap * tanh(score / cap) when cap > 0; running maximum and sum in float32; then every lane sums
// its columns of the values with the tile's weights. The result is divided by the sum and
// multiplied by sigmoid(gate) when a gate is given: a number per head, or one per column with
// `gate_wide`. With `sink` (H floats) the sum also holds exp(sink[h]), a term that has no key and no
// value and is not scaled. With `runs` the token also sees one key and value per run of `pool` tokens
// that ends at its position minus the window or before, in the same softmax, ahead of the tokens.
// With `score_bias` (H floats) there is no softmax: a key counts with sigmoid(score + score_bias[h]).
// With `chunk` the token sees the keys of its own stretch of `chunk` positions, counted from the sequence's
// first; the first `keep` keys are seen besides, ahead of the others.
#define Q3_CAP_DIM_MOST 512
#define Q3_CAP_VSLICES 8
template <typename TA>
__global__ void __launch_bounds__(64) softcap_attention_kernel(
    const TA* __restrict__ q, const TA* __restrict__ k_cache, const TA* __restrict__ v_cache,
    const int* __restrict__ block_table, int table_width, const int* __restrict__ seq_index,
    const int* __restrict__ positions, float scale, float cap, int window, int chunk, int keep, const float* __restrict__ gate,
    long gate_stride, int gate_wide, TA* __restrict__ out, int H, int G, int dim, int vdim, int page, int v_transposed,
    const float* __restrict__ sink, RunPlaces runs, const float* __restrict__ score_bias) {
  __shared__ float sq[Q3_CAP_DIM_MOST];
  __shared__ float sp[64];
  const int lane = threadIdx.x;
  const int t = blockIdx.x, h = blockIdx.y;
  const int g = h / (H / G);
  const int pos = positions[t];
  const TA* qr = q + ((size_t)t * H + h) * dim;
  for (int e = lane; e < dim; e += 64) sq[e] = to_float(qr[e]);
  __syncthreads();
  const bool weighed = score_bias != nullptr;          // sigmoids, not a softmax
  const float bias = weighed ? score_bias[h] : 0.f;
  float m = weighed ? 0.f : -INFINITY, l = 0.f;
  float acc[Q3_CAP_VSLICES];
#pragma unroll
  for (int i = 0; i < Q3_CAP_VSLICES; ++i) acc[i] = 0.f;
  // keys lo .. hi of one paged source
  auto walk = [&](const TA* ks, const TA* vs, const int* table, int lo, int hi) {
    for (int j0 = lo / 64 * 64; j0 <= hi; j0 += 64) {
      const int j = j0 + lane;
      const bool valid = j >= lo && j <= hi;
      float s = -INFINITY;
      if (valid) {
        const int pg = table[j / page];
        const TA* kr = ks + (((size_t)(pg < 0 ? 0 : pg) * G + g) * page + j % page) * dim;
        float dot = 0.f;
        for (int e = 0; e < dim; ++e) dot += sq[e] * to_float(kr[e]);
        s = dot * scale;
        if (cap > 0.f) s = cap * tanhf(s / cap);
      }
      float p;
      if (weighed) {
        p = valid ? 1.f / (1.f + expf(-(s + bias))) : 0.f;
      } else {
        const float m_new = fmaxf(m, wave_max(s));
        p = valid ? expf(s - m_new) : 0.f;
        const float keep = m == -INFINITY ? 0.f : expf(m - m_new);
        l = l * keep + wave_sum(p);
        m = m_new;
#pragma unroll
        for (int i = 0; i < Q3_CAP_VSLICES; ++i) acc[i] *= keep;
      }
      sp[lane] = p;
      __syncthreads();
      const int last = hi - j0 < 63 ? hi - j0 : 63;
      for (int jj = (lo > j0 ? lo - j0 : 0); jj <= last; ++jj) {
        const float pj = sp[jj];
        const int key = j0 + jj;
        const int pg = table[key / page];
        const size_t head = (size_t)(pg < 0 ? 0 : pg) * G + g;
        const TA* vr = v_transposed ? vs + head * vdim * page + key % page : vs + (head * page + key % page) * vdim;
        const int apart = v_transposed ? page : 1;
#pragma unroll
        for (int i = 0; i < Q3_CAP_VSLICES; ++i) {
          const int c = lane + 64 * i;
          if (c < vdim) acc[i] += pj * to_float(vr[(size_t)c * apart]);
        }
      }
      __syncthreads();
    }
  };
  if (runs.k && pos - window + 1 > 0) {
    const int seen = (pos - window + 1) / runs.pool;
    walk((const TA*)runs.k, (const TA*)runs.v, runs.table + (size_t)seq_index[t] * runs.width, 0, seen - 1);
  }
  const int* table = block_table + (size_t)seq_index[t] * table_width;
  const int lo = chunk > 0 ? pos - pos % chunk : (window > 0 ? max(0, pos - window + 1) : 0);
  if (keep > 0 && lo > 0) walk(k_cache, v_cache, table, 0, min(keep, lo) - 1);
  walk(k_cache, v_cache, table, lo, pos);
  if (sink) l += expf(sink[h] - m);
  const float norm = weighed ? 1.f : 1.f / l;
#pragma unroll
  for (int i = 0; i < Q3_CAP_VSLICES; ++i) {
    const int c = lane + 64 * i;
    if (c < vdim) {
      const float open = gate ? 1.f / (1.f + expf(-gate[(size_t)t * gate_stride + (gate_wide ? h * vdim + c : h)])) : 1.f;
      out[((size_t)t * H + h) * vdim + c] = from_float<TA>(acc[i] * (open * norm));
    }
  }
}

// Queries, keys and values with a norm per head: one block per token, a wavefront per head in turn.
// The row is [q: H dim | k: G dim | v: G vdim | ...] float32, or [q: H dim | ...] for a layer that
// makes no keys of its own (`G` 0). Every head of q (of k) is divided by its own root mean square
// and multiplied by `q_weight` (`k_weight`), dim numbers that all heads share; no rotation. q goes
// to `q_out`, k and v into the token's place in the cache.
template <typename TA>
__global__ void __launch_bounds__(256) headnorm_prepare_kernel(
    const float* __restrict__ rows, long row_stride, const float* __restrict__ q_weight,
    const float* __restrict__ k_weight, float eps, const int* __restrict__ positions, const int* __restrict__ seq_index,
    const int* __restrict__ block_table, int table_width, TA* __restrict__ k_cache, TA* __restrict__ v_cache, int page,
    TA* __restrict__ q_out, int H, int G, int dim, int vdim, int v_transposed) {
  const int t = blockIdx.x;
  const int wave = threadIdx.x / Q3_WAVE, lane = threadIdx.x % Q3_WAVE, waves = blockDim.x / Q3_WAVE;
  const float* row = rows + (size_t)t * row_stride;
  const int nq = H * dim, nk = G * dim;
  for (int h = wave; h < H; h += waves) {
    const float* src = row + (size_t)h * dim;
    float acc = 0.f;
    for (int e = lane; e < dim; e += Q3_WAVE) acc += src[e] * src[e];
    const float r = rsqrtf(wave_sum(acc) / (float)dim + eps);
    for (int e = lane; e < dim; e += Q3_WAVE) q_out[(size_t)t * nq + h * dim + e] = from_float<TA>(src[e] * r * q_weight[e]);
  }
  if (G == 0) return;
  const int pos = positions[t];
  const int pg = block_table[(size_t)seq_index[t] * table_width + pos / page];
  if (pg < 0) return;
  const int off = pos % page;
  for (int g = wave; g < G; g += waves) {
    const float* src = row + nq + (size_t)g * dim;
    float acc = 0.f;
    for (int e = lane; e < dim; e += Q3_WAVE) acc += src[e] * src[e];
    const float r = rsqrtf(wave_sum(acc) / (float)dim + eps);
    for (int e = lane; e < dim; e += Q3_WAVE)
      k_cache[(((size_t)pg * G + g) * page + off) * dim + e] = from_float<TA>(src[e] * r * k_weight[e]);
    const float* val = row + nq + nk + (size_t)g * vdim;
    for (int e = lane; e < vdim; e += Q3_WAVE) {
      const size_t at = v_transposed ? (((size_t)pg * G + g) * vdim + e) * page + off
                                     : (((size_t)pg * G + g) * page + off) * vdim + e;
      v_cache[at] = from_float<TA>(val[e]);
    }
  }
}

extern "C" int q3_headnorm_prepare(const float* rows, long row_stride, const float* q_weight, const float* k_weight,
                                   float eps, const int* positions, const int* seq_index, const int* block_table,
                                   int table_width, void* k_cache, void* v_cache, int page, void* q_out, int T, int H,
                                   int G, int dim, int vdim, int v_transposed, int act_dtype, hipStream_t stream) {
  if (T <= 0 || H <= 0 || G < 0 || dim <= 0 || vdim <= 0 || !q_weight) return Q3_ERR_BAD_ARGUMENT;
  if (G > 0 && (H % G || !k_weight || !k_cache || !v_cache || !block_table || page <= 0 || table_width <= 0))
    return Q3_ERR_BAD_ARGUMENT;
  Q3_DISPATCH_DTYPE(act_dtype, TA,
                    hipLaunchKernelGGL(headnorm_prepare_kernel<TA>, dim3(T), dim3(256), 0, stream, rows, row_stride,
                                       q_weight, k_weight, eps, positions, seq_index, block_table, table_width,
                                       (TA*)k_cache, (TA*)v_cache, page, (TA*)q_out, H, G, dim, vdim, v_transposed));
  return q3_launch_status();
}

// out[t, h, :] *= sigmoid(gate[t, h]) for a result that another kernel has left ungated; with `per` 1
// instead of vdim, a gate per column.
template <typename TA>
__global__ void gate_heads_kernel(TA* __restrict__ out, const float* __restrict__ gate, long gate_stride, int H, int vdim,
                                  int per) {
  const int t = blockIdx.x;
  for (int e = threadIdx.x; e < H * vdim; e += blockDim.x) {
    const float open = 1.f / (1.f + expf(-gate[(size_t)t * gate_stride + (per == 1 ? e : e / per)]));
    out[(size_t)t * H * vdim + e] = from_float<TA>(to_float(out[(size_t)t * H * vdim + e]) * open);
  }
}

extern "C" int q3_gate_heads(void* out, const float* gate, long gate_stride, int gate_wide, int T, int H, int vdim,
                             int act_dtype, hipStream_t stream) {
  if (T <= 0 || H <= 0 || vdim <= 0) return Q3_ERR_BAD_ARGUMENT;
  Q3_DISPATCH_DTYPE(act_dtype, TA, hipLaunchKernelGGL(gate_heads_kernel<TA>, dim3(T), dim3(256), 0, stream, (TA*)out,
                                                      gate, gate_stride, H, vdim, gate_wide ? 1 : vdim));
  return q3_launch_status();
}

extern "C" int q3_softcap_prepare(const float* rows, long row_stride, const float* bias, const float* q_weight,
                                  const float* k_weight, float eps, const float* inv_freq, int half,
                                  const int* positions, const int* seq_index, const int* block_table, int table_width,
                                  void* k_cache, void* v_cache, int page, void* q_out, int T, int H, int G, int dim,
                                  int vdim, int v_transposed, int act_dtype, hipStream_t stream) {
  if (T <= 0 || H <= 0 || G <= 0 || H % G || dim <= 0 || vdim <= 0 || half < 0 || 2 * half > dim) return Q3_ERR_BAD_ARGUMENT;
  if (half > 0 && !inv_freq) return Q3_ERR_BAD_ARGUMENT;
  if (k_cache && (!v_cache || !block_table || page <= 0 || table_width <= 0)) return Q3_ERR_BAD_ARGUMENT;
  Q3_DISPATCH_DTYPE(act_dtype, TA,
                    hipLaunchKernelGGL(softcap_prepare_kernel<TA>, dim3(T), dim3(256), 0, stream, rows, row_stride, bias,
                                       q_weight, k_weight, eps, inv_freq, half, positions, seq_index, block_table,
                                       table_width, (TA*)k_cache, (TA*)v_cache, page, (TA*)q_out, H, G, dim, vdim,
                                       v_transposed));
  return q3_launch_status();
}

// `run_k` null: no runs. `score_bias` null: a softmax.
extern "C" int q3_softcap_attention(const void* q, const void* k_cache, const void* v_cache, const int* block_table,
                                    int table_width, const int* seq_index, const int* positions, float scale, float cap,
                                    int window, int chunk, int keep, const float* gate, long gate_stride, int gate_wide, void* out, int T,
                                    int H, int G, int dim, int vdim, int page, int v_transposed, const float* sink,
                                    const void* run_k, const void* run_v, const int* run_table, int run_width, int pool,
                                    const float* score_bias, int act_dtype, hipStream_t stream) {
  if (T <= 0 || H <= 0 || G <= 0 || H % G || dim <= 0 || vdim <= 0 || page <= 0 || table_width <= 0 || window < 0 ||
      H > 65535)
    return Q3_ERR_BAD_ARGUMENT;
  if (run_k && (!run_v || !run_table || run_width <= 0 || pool <= 0 || window <= 0 || !v_transposed))
    return Q3_ERR_BAD_ARGUMENT;
  if (score_bias && (sink || run_k)) return Q3_ERR_BAD_ARGUMENT;
  if (chunk < 0 || keep < 0 || (chunk > 0 && window > 0) || (run_k && (chunk > 0 || keep > 0))) return Q3_ERR_BAD_ARGUMENT;
  if (dim > Q3_CAP_DIM_MOST || vdim > 64 * Q3_CAP_VSLICES) return Q3_ERR_UNSUPPORTED;
  const RunPlaces runs{const_cast<void*>(run_k), const_cast<void*>(run_v), run_table, run_width, pool};
  Q3_DISPATCH_DTYPE(act_dtype, TA,
                    hipLaunchKernelGGL(softcap_attention_kernel<TA>, dim3(T, H), dim3(64), 0, stream, (const TA*)q,
                                       (const TA*)k_cache, (const TA*)v_cache, block_table, table_width, seq_index,
                                       positions, scale, cap, window, chunk, keep, gate, gate_stride, gate_wide, (TA*)out, H, G, dim,
                                       vdim, page, v_transposed, sink, runs, score_bias));
  return q3_launch_status();
}
