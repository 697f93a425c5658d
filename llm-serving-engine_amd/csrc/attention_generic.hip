// Paged attention for any head size, in float32 arithmetic on float32 or bfloat16 pages.
// One block per (token, query head): the token's query attends to the cached keys of its
// request at positions (p - window, p], read through the request's block table, with an
// online softmax over tiles of 128 keys (reference model.py:140-175, the same recurrence per
// page).  It serves prompt portions and single decoded tokens alike: what differs between
// them is only how many tokens of a request are in the step.  This is the true 32-bit path
// and the path for head sizes without an MFMA kernel.
// Two things may change a score before the softmax, for position encodings and models that want
// them (the reference has neither): `soft_cap` > 0 squashes it to cap * tanh(score / cap), and
// `slopes` (one per query head) then adds -slope * (query position - key position), a bias that
// grows with distance.  With `sinks` (one per query head) the softmax's denominator has exp(sink) more, once, with
// no value to it: a key that is not there.  `chunk` > 0 is a mask instead of a window: a query sees the keys of its own chunk of
// so many positions, counted from the sequence's start.  `bias` (common.h: bias_element) is added to a score by the distance
// between query and key.  With `maps` = m > 1 a query row holds m maps side by side, each meets its own part of the keys and
// is an attention of its own: head h is map h % m of the queries' head h / m.
#include "common.h"

#define KEYS_PER_TILE 128
#define MAX_DIM 1024

template <typename T>
__global__ __launch_bounds__(KEYS_PER_TILE) void attention_generic_kernel(
    const T* __restrict__ qkv, int row_width, T* __restrict__ out, int out_stride, const T* __restrict__ keys,
    const T* __restrict__ values, const int* __restrict__ block_tables, int table_width,
    const int* __restrict__ token_sequence, const int* __restrict__ positions, int heads, int kv_heads, int dim,
    int page_size, float scale, int window, const float* __restrict__ slopes, float soft_cap, const float* __restrict__ sinks,
    int keep_first, int chunk, int maps, const float* __restrict__ bias, int reach) {
  __shared__ float query[MAX_DIM];
  __shared__ float weights[KEYS_PER_TILE];
  __shared__ float shared[17];
  const int token = blockIdx.x, head = blockIdx.y;
  const int kv_head = head / (heads / kv_heads);
  const int position = positions[token];
  const int* table = block_tables + (size_t)token_sequence[token] * table_width;
  const T* q = qkv + (size_t)token * row_width + head / maps * dim;
  const int of_map = dim / maps, map_first = head % maps * of_map;
  for (int d = threadIdx.x; d < dim; d += blockDim.x)
    query[d] = d >= map_first && d < map_first + of_map ? to_float(q[d]) * scale : 0.f;
  __syncthreads();

  const int first = chunk > 0 ? position - position % chunk : window > 0 ? max(0, position - window + 1) : 0;
  const float slope = slopes ? slopes[head] : 0.f;
  const int width = key_piece_width(dim);
  const int per_thread = (dim + KEYS_PER_TILE - 1) / KEYS_PER_TILE;  // output dims per thread, <= 4
  float acc[MAX_DIM / KEYS_PER_TILE] = {};
  float running_max = -INFINITY, running_sum = 0.f;

  // The keys a query sees, counted through: the sequence's first `kept` keys (those of its first `keep_first` that the
  // window has passed; they stay visible at their own positions), then the window's.
  const int kept = min(keep_first, first), seen = kept + position - first + 1;
  auto key_of = [&](int index) { return index < kept ? index : first + index - kept; };
  for (int tile = 0; tile < seen; tile += KEYS_PER_TILE) {
    const int key = key_of(tile + threadIdx.x);
    float score = -INFINITY;
    if (key <= position) {
      const int page = table[key / page_size];
      // the key's pieces lie page_size * width apart (common.h: key_element)
      const T* k = keys + ((size_t)page * kv_heads + kv_head) * page_size * dim + (size_t)(key % page_size) * width;
      float dot = 0.f;
      for (int piece = 0; piece < dim / width; ++piece) {
        const T* part = k + (size_t)piece * page_size * width;
        for (int e = 0; e < width; ++e) dot = fmaf(query[piece * width + e], to_float(part[e]), dot);
      }
      score = dot;
      if (soft_cap > 0.f) score = soft_cap * tanhf(score / soft_cap);
      score -= slope * (float)(position - key);
      if (bias) score += bias[(size_t)head * (reach + BIAS_SPARE) + bias_element(position - key, reach)];
    }
    const float tile_max = block_max(score, shared);
    const float next_max = fmaxf(running_max, tile_max);
    const float correction = expf(running_max - next_max);  // 0 on the first tile
    const float weight = key <= position ? expf(score - next_max) : 0.f;
    weights[threadIdx.x] = weight;
    const float tile_sum = block_sum(weight, shared);  // also orders the writes to `weights`
    running_sum = running_sum * correction + tile_sum;
    running_max = next_max;
    const int in_tile = min(KEYS_PER_TILE, seen - tile);
    for (int i = 0; i < per_thread; ++i) {
      const int d = threadIdx.x + i * KEYS_PER_TILE;
      if (d >= dim) break;
      float sum = 0.f;
      for (int j = 0; j < in_tile; ++j) {
        const int at = key_of(tile + j);
        const int page = table[at / page_size];
        const T* v = values + ((size_t)page * kv_heads + kv_head) * page_size * dim;
        sum = fmaf(weights[j], to_float(v[value_element(d, at % page_size, page_size, dim)]), sum);  // common.h: value_element
      }
      acc[i] = acc[i] * correction + sum;
    }
    __syncthreads();
  }
  float shrink = 1.f;  // what the results are multiplied by where the sink's exponential is the largest
  if (sinks) {
    const float sink = sinks[head], top = fmaxf(running_max, sink);
    shrink = expf(running_max - top);
    running_sum = running_sum * shrink + expf(sink - top);
  }
  T* o = out + (size_t)token * out_stride + head * dim;
  for (int i = 0; i < per_thread; ++i) {
    const int d = threadIdx.x + i * KEYS_PER_TILE;
    if (d < dim) o[d] = from_float<T>(acc[i] * shrink / running_sum);
  }
}

extern "C" int llmserve_attention_generic(const void* qkv, int row_width, void* out, int out_stride, int is_float, const void* keys,
                                          const void* values, const int* block_tables, int table_width,
                                          const int* token_sequence, const int* positions, int tokens, int heads,
                                          int kv_heads, int dim, int page_size, float scale, int window,
                                          const float* slopes, float soft_cap, const float* sinks, int keep_first,
                                          int chunk, int maps, const float* bias, int reach, hipStream_t stream) {
  if (tokens <= 0) return 0;
  if (dim > MAX_DIM || dim <= 0 || heads % kv_heads || page_size <= 0 || keep_first < 0 || chunk < 0 ||
      (chunk > 0 && (window > 0 || keep_first > 0)) || out_stride < heads * dim || maps < 1 || heads % maps || dim % maps ||
      (bias && reach < 1))
    return ERR_BAD_ARGUMENT;
  dim3 grid(tokens, heads);
  if (is_float)
    hipLaunchKernelGGL(attention_generic_kernel<float>, grid, dim3(KEYS_PER_TILE), 0, stream, (const float*)qkv,
                       row_width, (float*)out, out_stride, (const float*)keys, (const float*)values, block_tables, table_width,
                       token_sequence, positions, heads, kv_heads, dim, page_size, scale, window, slopes, soft_cap, sinks, keep_first, chunk,
                       maps, bias, reach);
  else
    hipLaunchKernelGGL(attention_generic_kernel<bf16_t>, grid, dim3(KEYS_PER_TILE), 0, stream, (const bf16_t*)qkv,
                       row_width, (bf16_t*)out, out_stride, (const bf16_t*)keys, (const bf16_t*)values, block_tables, table_width,
                       token_sequence, positions, heads, kv_heads, dim, page_size, scale, window, slopes, soft_cap, sinks, keep_first, chunk,
                       maps, bias, reach);
  return LAUNCH_STATUS();
}
