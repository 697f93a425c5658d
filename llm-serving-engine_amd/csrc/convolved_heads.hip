// Queries, keys and values of projected rows made ready for the attention:
//   convolved_heads    a causal convolution a channel (or none), then per query and key map an RMS norm with or without a
//                      weight (or none), a temperature of the queries by position, and rows of one head width; in a step
//                      of single tokens the keys and values also go to their pages and the convolutions' kept inputs move on
//   difference_heads   the results of two softmax maps a head put together: d = a1 - factor * a2, d / rms(d) * out_scale
//   gate_columns       rows times the sigmoid of other rows, element by element
// Everything is float32 arithmetic, rounded once.
#include "common.h"

#define MAX_TAPS 16

struct HeadRows {
  int x_width, q_first, k_first, v_first;  // where queries, keys and values begin in a row of x
  int heads, kv_heads, maps, dim, vdim;    // a query or key head is `maps` maps of `dim` side by side
  int width;                               // of a head in the rows written: map m at m * (width / maps), zeros elsewhere
  int norm;                                // maps are divided by their root mean square
  int taps, channels;                      // of the convolutions over x's first `channels` columns; taps 0: none
  float eps, temp_coef;
  int temp_every;                          // 0: no temperature
};

__device__ __forceinline__ float query_temperature(const HeadRows& z, int position) {
  return z.temp_every > 0 ? 1.f + z.temp_coef * logf((float)((position + 1) / z.temp_every) + 1.f) : 1.f;
}

// ---------------------------------------------------------------------------- any type and size
// One block per token, a wave a map at a time.
template <typename T>
__global__ __launch_bounds__(1024) void convolved_heads_kernel(const T* __restrict__ x, HeadRows z, const float* __restrict__ taps,
                                                               const float* __restrict__ window, const int* __restrict__ token_request,
                                                               const int* __restrict__ start, const int* __restrict__ slots,
                                                               const int* __restrict__ positions, const void* __restrict__ q_weight,
                                                               const void* __restrict__ k_weight, int weight_is_float,
                                                               T* __restrict__ out) {
  const int token = blockIdx.x;
  const T* row = x + (size_t)token * z.x_width;
  const int request = z.taps ? token_request[token] : 0;
  const int inside = z.taps ? token - start[request] : 0;  // the token's number within its request's share of the step
  const float* kept = z.taps > 1 ? window + (size_t)slots[request] * (z.taps - 1) * z.channels : nullptr;
  auto value_of = [&](int column) {
    if (z.taps == 0) return to_float(row[column]);
    float sum = 0.f;
    for (int j = 0; j < z.taps; ++j) {
      const int n = inside - (z.taps - 1) + j;
      const float v = n >= 0 ? to_float(row[column - (ptrdiff_t)(z.taps - 1 - j) * z.x_width]) : kept[(size_t)(z.taps - 1 + n) * z.channels + column];
      sum += taps[(size_t)column * z.taps + j] * v;
    }
    return sum;
  };
  T* dst = out + (size_t)token * (z.heads + 2 * z.kv_heads) * z.width;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, waves = blockDim.x >> 6;
  const int part = z.width / z.maps;
  const float temperature = query_temperature(z, positions ? positions[token] : 0);
  for (int unit = wave; unit < (z.heads + z.kv_heads) * z.maps; unit += waves) {
    const bool is_key = unit >= z.heads * z.maps;
    const int index = is_key ? unit - z.heads * z.maps : unit;
    const int first = (is_key ? z.k_first : z.q_first) + index * z.dim;
    const void* weight = is_key ? k_weight : q_weight;
    float scale = 1.f;
    if (z.norm) {
      float squares = 0.f;
      for (int e = lane; e < z.dim; e += WAVE) {
        const float v = value_of(first + e);
        squares += v * v;
      }
      scale = 1.f / sqrtf(wave_sum(squares) / (float)z.dim + z.eps);
    }
    T* to = dst + (size_t)unit * part;
    for (int e = lane; e < part; e += WAVE) {
      float result = 0.f;
      if (e < z.dim) {
        result = value_of(first + e) * scale;
        if (z.norm && weight) result *= load_as_float(weight, weight_is_float, e);
        if (!is_key) result *= temperature;
      }
      to[e] = from_float<T>(result);
    }
    for (int e = z.maps * part + lane; index % z.maps == z.maps - 1 && e < z.width; e += WAVE) (to - (z.maps - 1) * part)[e] = from_float<T>(0.f);
  }
  T* value_dst = dst + (size_t)(z.heads + z.kv_heads) * z.width;
  for (int index = threadIdx.x; index < z.kv_heads * z.width; index += blockDim.x) {
    const int head = index / z.width, e = index % z.width;
    value_dst[index] = from_float<T>(e < z.vdim ? value_of(z.v_first + head * z.vdim + e) : 0.f);
  }
}

// window[slot] <- the last taps - 1 inputs after this step: the step's own last ones, and before them (for a step of
// fewer tokens) the kept ones moved up.  One thread per (request, channel) reads all it needs before it writes.
template <typename T>
__global__ __launch_bounds__(256) void keep_inputs_kernel(const T* __restrict__ x, int x_width, int channels, int taps,
                                                          const int* __restrict__ start, const int* __restrict__ slots,
                                                          float* __restrict__ window) {
  const int c = blockIdx.y * blockDim.x + threadIdx.x;
  if (c >= channels) return;
  const int request = blockIdx.x, first = start[request], count = start[request + 1] - first;
  if (count <= 0) return;
  float* kept = window + (size_t)slots[request] * (taps - 1) * channels;
  float next[MAX_TAPS];
#pragma unroll
  for (int i = 0; i < MAX_TAPS; ++i) {
    if (i < taps - 1) {
      const int n = count - (taps - 1) + i;  // the step's token number that lands at place i
      next[i] = n >= 0 ? to_float(x[(size_t)(first + n) * x_width + c]) : kept[(size_t)(i + count) * channels + c];
    }
  }
#pragma unroll
  for (int i = 0; i < MAX_TAPS; ++i)
    if (i < taps - 1) kept[(size_t)i * channels + c] = next[i];
}

// ---------------------------------------------------------------------------- bfloat16 in 16-byte pieces
// Sizes that are multiples of 8.  A thread owns eight channels of a map (or of a value head) and takes them through
// `TOKENS` tokens in a row; a map's sum of squares is added up over the LANES lanes that hold its pieces (a power of two
// from width / maps / 8 on; those beyond the map write the zeros).  TAPS 0: no convolution.
// `keys` (a step of single tokens): the token's keys and values also go to their pages, and the kept inputs move on.
typedef bf16_t bf16x8 __attribute__((ext_vector_type(8)));

template <int TAPS, int TOKENS>
__global__ __launch_bounds__(256) void convolved_heads_vector_kernel(
    const bf16_t* __restrict__ x, HeadRows z, int lanes, const float* __restrict__ taps, float* __restrict__ window,
    const int* __restrict__ token_request, const int* __restrict__ start, const int* __restrict__ slots,
    const int* __restrict__ positions, const void* __restrict__ q_weight, const void* __restrict__ k_weight, int weight_is_float,
    bf16_t* __restrict__ out, int tokens, bf16_t* __restrict__ keys, bf16_t* __restrict__ values, const int* __restrict__ page_slots,
    int page_size, int keep_inputs) {
  const int part = z.width / z.maps, units = (z.heads + z.kv_heads) * z.maps;
  const int of_maps = units * lanes, all = of_maps + z.kv_heads * (z.width / 8);
  const int piece_index = blockIdx.y * blockDim.x + threadIdx.x;
  if (piece_index >= all) return;  // (the pieces of a map are all here or all beyond: `lanes` divides a wave)
  const bool is_value = piece_index >= of_maps;
  const int unit = is_value ? (piece_index - of_maps) / (z.width / 8) : piece_index / lanes;
  const int piece = is_value ? (piece_index - of_maps) % (z.width / 8) : piece_index % lanes;
  const bool is_key = !is_value && unit >= z.heads * z.maps;
  const int size = is_value ? z.vdim : z.dim;
  const bool live = piece * 8 < size;
  const int column = (is_value ? z.v_first + unit * z.vdim : is_key ? z.k_first + (unit - z.heads * z.maps) * z.dim : z.q_first + unit * z.dim) + piece * 8;
  const int to = is_value ? (z.heads + z.kv_heads + unit) * z.width + piece * 8 : unit * part + piece * 8;
  const bool writes = is_value || piece * 8 < part;
  const int out_width = (z.heads + 2 * z.kv_heads) * z.width;

  float tap[TAPS > 0 ? TAPS : 1][8];
  if constexpr (TAPS > 0) {
    float flat[TAPS * 8];  // [channel][tap]
    const float* from = taps + (size_t)(live ? column : 0) * TAPS;
#pragma unroll
    for (int i = 0; i < TAPS * 2; ++i) *(float4*)(flat + 4 * i) = *(const float4*)(from + 4 * i);
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) tap[j][e] = flat[e * TAPS + j];
  }
  float weight[8];
  const void* given = is_key ? k_weight : q_weight;
#pragma unroll
  for (int e = 0; e < 8; ++e) weight[e] = !is_value && z.norm && given && live ? load_as_float(given, weight_is_float, piece * 8 + e) : 1.f;

#pragma unroll
  for (int r = 0; r < TOKENS; ++r) {
    const int token = blockIdx.x * TOKENS + r;
    if (token >= tokens) return;  // (the same for the whole block)
    const bf16_t* row = x + (size_t)token * z.x_width + (live ? column : 0);
    float value[8];
    [[maybe_unused]] float* kept = nullptr;
    [[maybe_unused]] bf16x8 newest;
    if constexpr (TAPS == 0) {
      const bf16x8 raw = *(const bf16x8*)row;
#pragma unroll
      for (int e = 0; e < 8; ++e) value[e] = (float)raw[e];
    } else {
      // (a step of single tokens: token i is request i's, its first in the step)
      const int request = TOKENS == 1 ? token : token_request[token], inside = TOKENS == 1 ? 0 : token - start[request];
      if constexpr (TAPS > 1) kept = window + (size_t)slots[request] * (TAPS - 1) * z.channels + (live ? column : 0);
      float input[TAPS][8];
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        const int n = inside - (TAPS - 1) + j;
        if (n >= 0) {
          const bf16x8 raw = *(const bf16x8*)(row - (ptrdiff_t)(TAPS - 1 - j) * z.x_width);
#pragma unroll
          for (int e = 0; e < 8; ++e) input[j][e] = (float)raw[e];
        } else {
          const float* from = kept + (size_t)(TAPS - 1 + n) * z.channels;
          *(float4*)input[j] = *(const float4*)from;
          *(float4*)(input[j] + 4) = *(const float4*)(from + 4);
        }
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        value[e] = 0.f;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) value[e] += tap[j][e] * input[j][e];
      }
      if (TOKENS == 1 && keep_inputs && live) {  // (a step of single tokens: the inputs move up by one)
#pragma unroll
        for (int j = 1; j < TAPS; ++j) {
          float* at = kept + (size_t)(j - 1) * z.channels;
          *(float4*)at = *(const float4*)input[j];
          *(float4*)(at + 4) = *(const float4*)(input[j] + 4);
        }
      }
    }
    float scale = 1.f;
    if (z.norm && !is_value) {
      float squares = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) squares += live ? value[e] * value[e] : 0.f;
      for (int offset = lanes / 2; offset > 0; offset >>= 1) squares += __shfl_xor(squares, offset, WAVE);
      scale = 1.f / sqrtf(squares / (float)z.dim + z.eps);
    }
    if (!is_value && !is_key && z.temp_every > 0) scale *= query_temperature(z, positions[token]);
    bf16x8 result;
#pragma unroll
    for (int e = 0; e < 8; ++e) result[e] = (bf16_t)(live ? value[e] * scale * weight[e] : 0.f);
    if (writes) *(bf16x8*)(out + (size_t)token * out_width + to) = result;
    if (keys && writes && (is_value || is_key)) {
      const int slot = page_slots[token];
      if (slot >= 0) {
        const int page = slot / page_size, offset = slot % page_size;
        if (is_value) {
          bf16_t* block = values + ((size_t)page * z.kv_heads + unit) * page_size * z.width;
#pragma unroll
          for (int e = 0; e < 8; ++e) block[value_element(piece * 8 + e, offset, page_size, z.width)] = result[e];
        } else {
          const int head = (unit - z.heads * z.maps) / z.maps, map = (unit - z.heads * z.maps) % z.maps;
          bf16_t* block = keys + ((size_t)page * z.kv_heads + head) * page_size * z.width;
          *(bf16x8*)(block + key_element(map * part + piece * 8, offset, page_size, z.width)) = result;
        }
      }
    }
  }
}

// `window` float32 [slots, taps - 1, channels] (taps > 1).  `single`: every request of the step brings one token; then (and
// only then) the keys and values may be stored here too (`keys` not null), by the kernel for sizes that come in pieces of
// eight, which `llmserve_convolved_heads_stores` tells.
static bool in_pieces(const HeadRows& z, int is_float) {
  return !is_float && z.dim % 8 == 0 && z.vdim % 8 == 0 && z.width % 8 == 0 && z.width % z.maps == 0 && (z.width / z.maps) % 8 == 0 &&
         z.width / z.maps <= 8 * WAVE && z.x_width % 8 == 0 && z.q_first % 8 == 0 && z.k_first % 8 == 0 && z.v_first % 8 == 0 &&
         z.taps <= 4 && z.channels % 4 == 0;
}

extern "C" int llmserve_convolved_heads_stores(int is_float, int x_width, int q_first, int k_first, int v_first, int maps, int dim,
                                               int vdim, int width, int taps, int channels) {
  const HeadRows z = {x_width, q_first, k_first, v_first, 1, 1, maps, dim, vdim, width, 1, taps, channels, 0.f, 0.f, 0};
  return in_pieces(z, is_float) ? 1 : 0;
}

extern "C" int llmserve_convolved_heads(const void* x, int is_float, int tokens, int x_width, int q_first, int k_first, int v_first,
                                        int heads, int kv_heads, int maps, int dim, int vdim, int width, int norm, float eps,
                                        const void* q_weight, const void* k_weight, int weight_is_float, const float* taps,
                                        int tap_count, int channels, float* window, const int* token_request, const int* start,
                                        const int* slots, int requests, const int* positions, float temp_coef, int temp_every,
                                        void* out, int single, void* keys, void* values, const int* page_slots, int page_size,
                                        hipStream_t stream) {
  if (tokens <= 0) return 0;
  if (heads < 1 || kv_heads < 0 || maps < 1 || dim < 1 || vdim < 1 || width % maps || width / maps < dim || width < vdim || q_first < 0 ||
      k_first < 0 || v_first < 0 || q_first + heads * maps * dim > x_width || k_first + kv_heads * maps * dim > x_width ||
      v_first + kv_heads * vdim > x_width || tap_count < 0 || tap_count > MAX_TAPS || (tap_count > 0 && (!taps || !token_request || !start)) ||
      (tap_count > 1 && (!window || !slots)) || temp_every < 0 || (temp_every > 0 && !positions))
    return ERR_BAD_ARGUMENT;
  if (tap_count > 0 && (channels < 1 || channels > x_width || q_first + heads * maps * dim > channels ||
                        (kv_heads > 0 && (k_first + kv_heads * maps * dim > channels || v_first + kv_heads * vdim > channels))))
    return ERR_BAD_ARGUMENT;
  const HeadRows z = {x_width, q_first, k_first, v_first, heads, kv_heads, maps, dim, vdim, width, norm, tap_count, channels, eps, temp_coef, temp_every};
  const bool pieces = in_pieces(z, is_float);
  if (keys && (!pieces || !single || !values || !page_slots || page_size < 1 || kv_heads < 1)) return ERR_BAD_ARGUMENT;
  bool kept = tap_count <= 1;  // nothing to keep, or kept by the first kernel
  if (pieces) {
    int lanes = 1;
    while (lanes * 8 < width / maps) lanes *= 2;
    const int all = (heads + kv_heads) * maps * lanes + kv_heads * (width / 8);
    const int threads = all <= 64 ? 64 : all <= 128 ? 128 : 256;
    const int run = single ? 1 : 4;
    const dim3 grid((tokens + run - 1) / run, (all + threads - 1) / threads);
#define LAUNCH_PIECES(TAPS, TOKENS)                                                                                            \
  hipLaunchKernelGGL((convolved_heads_vector_kernel<TAPS, TOKENS>), grid, dim3(threads), 0, stream, (const bf16_t*)x, z, lanes, taps, \
                     window, token_request, start, slots, positions, q_weight, k_weight, weight_is_float, (bf16_t*)out, tokens,     \
                     (bf16_t*)keys, (bf16_t*)values, page_slots, page_size, single)
    if (single) {
      switch (tap_count) {
        case 0: LAUNCH_PIECES(0, 1); break;
        case 1: LAUNCH_PIECES(1, 1); break;
        case 2: LAUNCH_PIECES(2, 1); break;
        case 3: LAUNCH_PIECES(3, 1); break;
        default: LAUNCH_PIECES(4, 1); break;
      }
      kept = true;
    } else {
      switch (tap_count) {
        case 0: LAUNCH_PIECES(0, 4); break;
        case 1: LAUNCH_PIECES(1, 4); break;
        case 2: LAUNCH_PIECES(2, 4); break;
        case 3: LAUNCH_PIECES(3, 4); break;
        default: LAUNCH_PIECES(4, 4); break;
      }
    }
#undef LAUNCH_PIECES
  } else {
    const int threads = WAVE * max(4, min(16, (heads + kv_heads) * maps));
    if (is_float)
      hipLaunchKernelGGL(convolved_heads_kernel<float>, dim3(tokens), dim3(threads), 0, stream, (const float*)x, z, taps, window,
                         token_request, start, slots, positions, q_weight, k_weight, weight_is_float, (float*)out);
    else
      hipLaunchKernelGGL(convolved_heads_kernel<bf16_t>, dim3(tokens), dim3(threads), 0, stream, (const bf16_t*)x, z, taps, window,
                         token_request, start, slots, positions, q_weight, k_weight, weight_is_float, (bf16_t*)out);
  }
  int status = LAUNCH_STATUS();
  if (status != 0 || kept) return status;
  const int threads = channels <= 64 ? 64 : channels <= 128 ? 128 : 256;
  const dim3 per_request(requests, (channels + threads - 1) / threads);
  if (is_float)
    hipLaunchKernelGGL(keep_inputs_kernel<float>, per_request, dim3(threads), 0, stream, (const float*)x, x_width, channels, tap_count, start,
                       slots, window);
  else
    hipLaunchKernelGGL(keep_inputs_kernel<bf16_t>, per_request, dim3(threads), 0, stream, (const bf16_t*)x, x_width, channels, tap_count,
                       start, slots, window);
  return LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------- two maps put together
// a: rows of heads * 2 results of `width`, [map 1 | map 2] head by head; out: rows of heads * vdim.  A wave a head.
template <typename T>
__global__ __launch_bounds__(256) void difference_heads_kernel(const T* __restrict__ a, T* __restrict__ out, int pairs, int width, int vdim,
                                                               float factor, float eps, float out_scale) {
  const int pair = blockIdx.x * (blockDim.x / WAVE) + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (pair >= pairs) return;
  const T* one = a + (size_t)pair * 2 * width;
  float squares = 0.f;
  for (int e = lane; e < vdim; e += WAVE) {
    const float d = to_float(one[e]) - factor * to_float(one[width + e]);
    squares += d * d;
  }
  const float scale = out_scale / sqrtf(wave_sum(squares) / (float)vdim + eps);
  for (int e = lane; e < vdim; e += WAVE)
    out[(size_t)pair * vdim + e] = from_float<T>((to_float(one[e]) - factor * to_float(one[width + e])) * scale);
}

extern "C" int llmserve_difference_heads(const void* a, int is_float, void* out, int tokens, int heads, int width, int vdim, float factor,
                                         float eps, float out_scale, hipStream_t stream) {
  if (tokens <= 0) return 0;
  if (heads < 1 || vdim < 1 || width < vdim) return ERR_BAD_ARGUMENT;
  const int pairs = tokens * heads;
  const dim3 grid((pairs + 3) / 4);
  if (is_float)
    hipLaunchKernelGGL(difference_heads_kernel<float>, grid, dim3(256), 0, stream, (const float*)a, (float*)out, pairs, width, vdim, factor,
                       eps, out_scale);
  else
    hipLaunchKernelGGL(difference_heads_kernel<bf16_t>, grid, dim3(256), 0, stream, (const bf16_t*)a, (bf16_t*)out, pairs, width, vdim,
                       factor, eps, out_scale);
  return LAUNCH_STATUS();
}

// ---------------------------------------------------------------------------- rows times the sigmoid of other rows
// out[t][h * vdim + e] = x[t][h * width + e] * sigmoid(gates[t][gate_first + h * vdim + e]), or, without gates, x alone: heads
// of `width` brought to `vdim` side by side.
template <typename T>
__global__ __launch_bounds__(256) void gate_columns_kernel(const T* __restrict__ x, int x_width, T* __restrict__ out, int out_width,
                                                           int heads, int width, int vdim, const T* __restrict__ gates, int gate_stride,
                                                           int gate_first, size_t count) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= count) return;
  const size_t token = i / ((size_t)heads * vdim);
  const int column = (int)(i % ((size_t)heads * vdim)), head = column / vdim, e = column % vdim;
  float v = to_float(x[token * x_width + head * width + e]);
  if (gates) v /= 1.f + expf(-to_float(gates[token * gate_stride + gate_first + column]));
  out[token * out_width + column] = from_float<T>(v);
}

extern "C" int llmserve_gate_columns(const void* x, int is_float, int x_width, void* out, int out_width, int tokens, int heads, int width,
                                     int vdim, const void* gates, int gate_stride, int gate_first, hipStream_t stream) {
  if (tokens <= 0) return 0;
  if (heads < 1 || vdim < 1 || width < vdim || x_width < heads * width || out_width < heads * vdim ||
      (gates && (gate_first < 0 || gate_first + heads * vdim > gate_stride)))
    return ERR_BAD_ARGUMENT;
  const size_t count = (size_t)tokens * heads * vdim;
  const dim3 grid((unsigned)((count + 255) / 256));
  if (is_float)
    hipLaunchKernelGGL(gate_columns_kernel<float>, grid, dim3(256), 0, stream, (const float*)x, x_width, (float*)out, out_width, heads,
                       width, vdim, (const float*)gates, gate_stride, gate_first, count);
  else
    hipLaunchKernelGGL(gate_columns_kernel<bf16_t>, grid, dim3(256), 0, stream, (const bf16_t*)x, x_width, (bf16_t*)out, out_width, heads,
                       width, vdim, (const bf16_t*)gates, gate_stride, gate_first, count);
  return LAUNCH_STATUS();
}
