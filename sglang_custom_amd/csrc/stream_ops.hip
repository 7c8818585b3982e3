// Kernels around a 32-bit residual stream whose sequences carry state from step to step:
//   * token + hashed-bigram embedding (the previous token of a sequence is state),
//   * weight-only layer norm fused with the token shift (the previous token's normed row is state),
//   * the layer norm of a sublayer's output, its sum into the stream and the layer norm in front of the next sublayer as one
//     launch,
//   * the commit of a step's new state rows,
//   * tanh-GELU-and-mul, and the sigmoid-gated residual update.
// Every reduction, normalisation, gate and the residual sum run in fp32 whatever the activation dtype T is;
// T only names what the GEMMs around these kernels read and write.
//
// Batch description shared by the kernels (all device pointers):
//   tok_req[t]    index b of token t's sequence in the batch        (null: b = t, every token is its own segment)
//   seg_start[b]  first token of b's segment in the flat token list (null with tok_req)
//   seg_len[b]    number of tokens of b in this step
//   positions[t]  position of token t in its sequence
//   req_pool_indices[b] -> req_to_state[.] = the sequence's state slot
#include "common.cuh"

#include <algorithm>

namespace mi355 {
namespace {

struct Seg {
  int b;
  bool first, last;
};
__device__ __forceinline__ Seg segment_of(int64_t t, const int32_t* tok_req, const int32_t* seg_start, const int32_t* seg_len) {
  Seg s;
  if (tok_req == nullptr) {
    s.b = (int)t;
    s.first = s.last = true;
  } else {
    s.b = tok_req[t];
    const int64_t t0 = seg_start[s.b];
    s.first = t == t0;
    s.last = t == t0 + seg_len[s.b] - 1;
  }
  return s;
}

// (x - mean) / sqrt(var + eps) of one row into buf (LDS, D floats); var = mean of squared deviations.  Every thread
// touches the same elements in all three passes, so buf needs no barrier of its own.  W = 4: four floats per access
// (D a multiple of 4, rows 16-byte aligned).
template <int W>
__device__ __forceinline__ void ln_row(float* buf, const float* __restrict__ x, int64_t D, float eps, float* red) {
  float s = 0.f;
  for (int64_t i = W * threadIdx.x; i < D; i += W * blockDim.x) {
    if constexpr (W == 4) {
      const float4 v = *reinterpret_cast<const float4*>(x + i);
      *reinterpret_cast<float4*>(buf + i) = v;
      s += (v.x + v.y) + (v.z + v.w);
    } else {
      const float v = x[i];
      buf[i] = v;
      s += v;
    }
  }
  const float mean = block_sum(s, red) / (float)D;
  float q = 0.f;
  for (int64_t i = W * threadIdx.x; i < D; i += W * blockDim.x) {
#pragma unroll
    for (int k = 0; k < W; ++k) {
      const float d = buf[i + k] - mean;
      q += d * d;
    }
  }
  const float var = block_sum(q, red) / (float)D;
  const float inv = 1.0f / sqrtf(var + eps);
  for (int64_t i = W * threadIdx.x; i < D; i += W * blockDim.x) {
#pragma unroll
    for (int k = 0; k < W; ++k) buf[i + k] = (buf[i + k] - mean) * inv;
  }
}

// One workgroup per token.  h = LN(x[t]) * w;  with `mu`: hs = h + (h_prev - h) * mu, where h_prev is the same
// quantity of the previous token: zero at position 0, the state row when t opens its segment, else recomputed from
// x[t - 1].  The last token of every segment leaves its fp32 h in h_last[b] for the commit kernel.
template <typename T, int W>
__global__ __launch_bounds__(256) void layernorm_shift_kernel(
    T* __restrict__ h_out, T* __restrict__ hs_out, float* __restrict__ h_last, const float* __restrict__ x,
    const T* __restrict__ w, const T* __restrict__ mu, const float* __restrict__ state, const int32_t* __restrict__ req_to_state,
    const int64_t* __restrict__ req_pool_indices, const int32_t* __restrict__ tok_req, const int32_t* __restrict__ seg_start,
    const int32_t* __restrict__ seg_len, const int64_t* __restrict__ positions, int64_t D, float eps) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ float red[16];
  float* cur = sm;
  float* prv = sm + D;
  const int64_t t = blockIdx.x;
  const int64_t i0 = W * threadIdx.x, step = W * blockDim.x;
  ln_row<W>(cur, x + t * D, D, eps, red);
  if (mu == nullptr) {
    for (int64_t i = i0; i < D; i += step) {
      Vec<T, W> o;
#pragma unroll
      for (int k = 0; k < W; ++k) o.v[k] = from_f32<T>(cur[i + k] * to_f32(w[i + k]));
      stvec<T, W>(h_out + t * D + i, o);
    }
    return;
  }
  const Seg sg = segment_of(t, tok_req, seg_start, seg_len);
  const int64_t pos = positions[t];
  if (pos == 0) {
    for (int64_t i = i0; i < D; i += step)
#pragma unroll
      for (int k = 0; k < W; ++k) prv[i + k] = 0.f;
  } else if (sg.first) {
    const float* srow = state + (int64_t)req_to_state[req_pool_indices[sg.b]] * D;
    for (int64_t i = i0; i < D; i += step)
#pragma unroll
      for (int k = 0; k < W; ++k) prv[i + k] = srow[i + k];
  } else {
    ln_row<W>(prv, x + (t - 1) * D, D, eps, red);
    for (int64_t i = i0; i < D; i += step)
#pragma unroll
      for (int k = 0; k < W; ++k) prv[i + k] *= to_f32(w[i + k]);
  }
  const bool keep = sg.last && h_last != nullptr;
  for (int64_t i = i0; i < D; i += step) {
    Vec<T, W> ho, so;
#pragma unroll
    for (int k = 0; k < W; ++k) {
      const float h = cur[i + k] * to_f32(w[i + k]);
      ho.v[k] = from_f32<T>(h);
      so.v[k] = from_f32<T>(h + (prv[i + k] - h) * to_f32(mu[i + k]));
      if (keep) h_last[(int64_t)sg.b * D + i + k] = h;
    }
    stvec<T, W>(h_out + t * D + i, ho);
    stvec<T, W>(hs_out + t * D + i, so);
  }
}

// One workgroup per token:  x[t] += N(b) * w_out,  h[t] = N(x[t]) * w_next  (w_next null: h[t] = x[t], h null: nothing), with
// b = sum_j coef[t][j] * y[rows[t][j]] (coef null: 1; rows null: y[t]) + sigmoid(gate[t]) * y2[t] (y2 null: nothing); N the layer
// norm, or (RMS) the division by the root mean square.  KEEP > 0: the row stays in
// registers, KEEP groups of eight features per thread (D <= 2048 KEEP, 16-byte accesses); KEEP 0: any D, the row in LDS.
struct LnAddParams {
  float* x;
  void* h;
  const void* y;
  const int32_t* rows;
  const float* coef;
  const void* y2;
  const float* gate;
  const void* w_out;
  const void* w_next;
  int64_t y_stride, y2_stride, gate_stride, D;
  int n_rows;
  float eps;
};

template <typename T> __device__ __forceinline__ void ld8f(const T* p, float* o) {
  if constexpr (sizeof(T) == 2) {
    const Vec<T, 8> v = ldvec<T, 8>(p);
#pragma unroll
    for (int k = 0; k < 8; ++k) o[k] = to_f32(v.v[k]);
  } else {
    const Vec<T, 4> a = ldvec<T, 4>(p), b = ldvec<T, 4>(p + 4);
#pragma unroll
    for (int k = 0; k < 4; ++k) { o[k] = to_f32(a.v[k]); o[4 + k] = to_f32(b.v[k]); }
  }
}
template <typename T> __device__ __forceinline__ void st8f(T* p, const float* o) {
  if constexpr (sizeof(T) == 2) {
    Vec<T, 8> v;
#pragma unroll
    for (int k = 0; k < 8; ++k) v.v[k] = from_f32<T>(o[k]);
    stvec<T, 8>(p, v);
  } else {
    Vec<T, 4> a, b;
#pragma unroll
    for (int k = 0; k < 4; ++k) { a.v[k] = from_f32<T>(o[k]); b.v[k] = from_f32<T>(o[4 + k]); }
    stvec<T, 4>(p, a);
    stvec<T, 4>(p + 4, b);
  }
}

// (v - mean) / sqrt(var + eps), or (RMS) v / sqrt(mean v^2 + eps), of a row held as G groups of eight per thread (groups past D
// hold zeros)
template <int G, bool RMS>
__device__ __forceinline__ void ln_regs(float (&v)[G][8], int64_t D, float eps, float* red) {
  if constexpr (RMS) {
    float q = 0.f;
#pragma unroll
    for (int g = 0; g < G; ++g)
#pragma unroll
      for (int k = 0; k < 8; ++k) q += v[g][k] * v[g][k];
    const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)D + eps);
#pragma unroll
    for (int g = 0; g < G; ++g)
#pragma unroll
      for (int k = 0; k < 8; ++k) v[g][k] *= inv;
    return;
  }
  float s = 0.f;
#pragma unroll
  for (int g = 0; g < G; ++g)
#pragma unroll
    for (int k = 0; k < 8; ++k) s += v[g][k];
  const float mean = block_sum(s, red) / (float)D;
  float q = 0.f;
#pragma unroll
  for (int g = 0; g < G; ++g) {
    const bool live = 8 * ((int64_t)threadIdx.x + 256 * g) < D;
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const float d = live ? v[g][k] - mean : 0.f;
      v[g][k] = d;
      q += d * d;
    }
  }
  const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)D + eps);
#pragma unroll
  for (int g = 0; g < G; ++g)
#pragma unroll
    for (int k = 0; k < 8; ++k) v[g][k] *= inv;
}

// the same of a row in LDS, in place; every thread touches the same elements in all passes
template <bool RMS>
__device__ __forceinline__ void ln_lds(float* buf, int64_t D, float eps, float* red) {
  float mean = 0.f;
  if constexpr (!RMS) {
    float s = 0.f;
    for (int64_t i = threadIdx.x; i < D; i += 256) s += buf[i];
    mean = block_sum(s, red) / (float)D;
  }
  float q = 0.f;
  for (int64_t i = threadIdx.x; i < D; i += 256) {
    const float d = buf[i] - mean;
    q += d * d;
  }
  const float inv = 1.0f / sqrtf(block_sum(q, red) / (float)D + eps);
  for (int64_t i = threadIdx.x; i < D; i += 256) buf[i] = (buf[i] - mean) * inv;
}

template <typename T, int KEEP, bool RMS>
__global__ __launch_bounds__(256) void layernorm_residual_add_kernel(const LnAddParams p) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x, D = p.D;
  float* xr = p.x + t * D;
  const T* y = static_cast<const T*>(p.y);
  const T* y2 = static_cast<const T*>(p.y2);
  const T* w_out = static_cast<const T*>(p.w_out);
  const T* w_next = static_cast<const T*>(p.w_next);
  T* h = static_cast<T*>(p.h) + t * D;
  const float sg = y2 != nullptr ? 1.0f / (1.0f + expf(-p.gate[t * p.gate_stride])) : 0.f;
  if constexpr (KEEP > 0) {
    float v[KEEP][8];
#pragma unroll
    for (int g = 0; g < KEEP; ++g) {
      const int64_t i = 8 * ((int64_t)threadIdx.x + 256 * g);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[g][k] = 0.f;
      if (i >= D) continue;
      if (p.rows == nullptr) {
        ld8f<T>(y + t * p.y_stride + i, v[g]);
      } else {
        for (int j = 0; j < p.n_rows; ++j) {      // fixed order: the sum does not depend on where the rows lie
          float e[8];
          ld8f<T>(y + (int64_t)p.rows[t * p.n_rows + j] * p.y_stride + i, e);
          const float c = p.coef != nullptr ? p.coef[t * p.n_rows + j] : 1.0f;
#pragma unroll
          for (int k = 0; k < 8; ++k) v[g][k] += c * e[k];
        }
      }
      if (y2 != nullptr) {
        float e[8];
        ld8f<T>(y2 + t * p.y2_stride + i, e);
#pragma unroll
        for (int k = 0; k < 8; ++k) v[g][k] += sg * e[k];
      }
    }
    ln_regs<KEEP, RMS>(v, D, p.eps, red);
#pragma unroll
    for (int g = 0; g < KEEP; ++g) {
      const int64_t i = 8 * ((int64_t)threadIdx.x + 256 * g);
      if (i >= D) continue;
      float w[8], r[8];
      ld8f<T>(w_out + i, w);
      ld8f<float>(xr + i, r);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[g][k] = r[k] + v[g][k] * w[k];
      st8f<float>(xr + i, v[g]);
      if (w_next == nullptr && p.h != nullptr) st8f<T>(h + i, v[g]);
    }
    if (w_next == nullptr) return;
    ln_regs<KEEP, RMS>(v, D, p.eps, red);
#pragma unroll
    for (int g = 0; g < KEEP; ++g) {
      const int64_t i = 8 * ((int64_t)threadIdx.x + 256 * g);
      if (i >= D) continue;
      float w[8];
      ld8f<T>(w_next + i, w);
#pragma unroll
      for (int k = 0; k < 8; ++k) w[k] *= v[g][k];
      st8f<T>(h + i, w);
    }
  } else {
    extern __shared__ __attribute__((aligned(16))) float sm[];      // [D]; a thread touches the same elements in every pass
    for (int64_t i = threadIdx.x; i < D; i += 256) {
      float b = 0.f;
      if (p.rows == nullptr) {
        b = to_f32(y[t * p.y_stride + i]);
      } else {
        for (int j = 0; j < p.n_rows; ++j) {
          const float c = p.coef != nullptr ? p.coef[t * p.n_rows + j] : 1.0f;
          b += c * to_f32(y[(int64_t)p.rows[t * p.n_rows + j] * p.y_stride + i]);
        }
      }
      if (y2 != nullptr) b += sg * to_f32(y2[t * p.y2_stride + i]);
      sm[i] = b;
    }
    ln_lds<RMS>(sm, D, p.eps, red);
    for (int64_t i = threadIdx.x; i < D; i += 256) {
      const float r = xr[i] + sm[i] * to_f32(w_out[i]);
      xr[i] = r;
      sm[i] = r;
      if (w_next == nullptr && p.h != nullptr) h[i] = from_f32<T>(r);
    }
    if (w_next == nullptr) return;
    ln_lds<RMS>(sm, D, p.eps, red);
    for (int64_t i = threadIdx.x; i < D; i += 256) h[i] = from_f32<T>(sm[i] * to_f32(w_next[i]));
  }
}

// One workgroup per token, the start of a pass over looped layers:  x[t] = y[t] + table[ids[t]] + step,  h[t] = N(x[t]) * w_next, N
// the division by the root mean square.  KEEP as above.
struct PassEntryParams {
  float* x;
  void* h;
  const void* y;
  const float* table;
  const int64_t* ids;
  const float* step;
  const void* w_next;
  int64_t y_stride, D, vocab;
  float eps;
};

template <typename T, int KEEP>
__global__ __launch_bounds__(256) void pass_entry_kernel(const PassEntryParams p) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x, D = p.D;
  int64_t id = p.ids[t];
  id = id < 0 ? 0 : (id >= p.vocab ? p.vocab - 1 : id);
  float* xr = p.x + t * D;
  const T* y = static_cast<const T*>(p.y) + t * p.y_stride;
  const float* tab = p.table + id * D;
  const T* w = static_cast<const T*>(p.w_next);
  T* h = static_cast<T*>(p.h) + t * D;
  if constexpr (KEEP > 0) {
    float v[KEEP][8];
#pragma unroll
    for (int g = 0; g < KEEP; ++g) {
      const int64_t i = 8 * ((int64_t)threadIdx.x + 256 * g);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[g][k] = 0.f;
      if (i >= D) continue;
      float e[8], s[8];
      ld8f<T>(y + i, v[g]);
      ld8f<float>(tab + i, e);
      ld8f<float>(p.step + i, s);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[g][k] += e[k] + s[k];
      st8f<float>(xr + i, v[g]);
    }
    ln_regs<KEEP, true>(v, D, p.eps, red);
#pragma unroll
    for (int g = 0; g < KEEP; ++g) {
      const int64_t i = 8 * ((int64_t)threadIdx.x + 256 * g);
      if (i >= D) continue;
      float e[8];
      ld8f<T>(w + i, e);
#pragma unroll
      for (int k = 0; k < 8; ++k) e[k] *= v[g][k];
      st8f<T>(h + i, e);
    }
  } else {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    for (int64_t i = threadIdx.x; i < D; i += 256) {
      const float r = to_f32(y[i]) + tab[i] + p.step[i];
      xr[i] = r;
      sm[i] = r;
    }
    ln_lds<true>(sm, D, p.eps, red);
    for (int64_t i = threadIdx.x; i < D; i += 256) h[i] = from_f32<T>(sm[i] * to_f32(w[i]));
  }
}

// x[t] = table[id] * scale + bigram[(prev * mul_prev + id * mul_cur) mod buckets]; row `buckets` at position 0.
template <typename T>
__global__ __launch_bounds__(256) void bigram_embedding_kernel(
    float* __restrict__ x, const int64_t* __restrict__ ids, const T* __restrict__ table, const T* __restrict__ bigram,
    const int32_t* __restrict__ prev_token, const int32_t* __restrict__ req_to_state, const int64_t* __restrict__ req_pool_indices,
    const int32_t* __restrict__ tok_req, const int32_t* __restrict__ seg_start, const int32_t* __restrict__ seg_len,
    const int64_t* __restrict__ positions, int64_t D, int64_t vocab, float scale, int64_t mul_prev, int64_t mul_cur,
    int64_t buckets) {
  const int64_t t = blockIdx.x;
  int64_t id = ids[t];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const Seg sg = segment_of(t, tok_req, seg_start, seg_len);
  int64_t row = buckets;
  if (positions[t] != 0) {
    int64_t prev;
    if (sg.first)
      prev = prev_token[req_to_state[req_pool_indices[sg.b]]];
    else
      prev = ids[t - 1];
    row = (prev * mul_prev + id * mul_cur) % buckets;
    if (row < 0) row += buckets;
  }
  const T* e = table + id * D;
  const T* g = bigram + row * D;
  for (int64_t i = threadIdx.x; i < D; i += blockDim.x) x[t * D + i] = to_f32(e[i]) * scale + to_f32(g[i]);
}

// grid (B, L): state[l][slot(b)] = h_last[l][b]; layer 0's workgroups also store the segment's last token id.
__global__ __launch_bounds__(256) void commit_state_kernel(
    float* __restrict__ state, int32_t* __restrict__ prev_token, const float* __restrict__ h_last, const int64_t* __restrict__ ids,
    const int32_t* __restrict__ req_to_state, const int64_t* __restrict__ req_pool_indices, const int32_t* __restrict__ seg_start,
    const int32_t* __restrict__ seg_len, int64_t B, int64_t D, int64_t state_layer_stride) {
  const int64_t b = blockIdx.x, l = blockIdx.y;
  const int64_t slot = req_to_state[req_pool_indices[b]];
  const float* src = h_last + (l * B + b) * D;
  float* dst = state + l * state_layer_stride + slot * D;
  for (int64_t i = threadIdx.x; i < D; i += blockDim.x) dst[i] = src[i];
  if (l == 0 && threadIdx.x == 0 && prev_token != nullptr) {
    const int64_t last = seg_start ? (int64_t)seg_start[b] + seg_len[b] - 1 : b;
    prev_token[slot] = (int32_t)ids[last];
  }
}

__device__ __forceinline__ float gelu_tanh_f(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

// out[t][i] = gelu_tanh(gate[t][i]) * up[t][i], 16 bytes of each operand per thread (d and the row stride multiples of the
// vector length, pointers 16-byte aligned)
template <typename T>
__global__ __launch_bounds__(256) void gelu_tanh_and_mul_vec_kernel(T* __restrict__ out, const T* __restrict__ gate, const T* __restrict__ up,
                                                                   int64_t rows, int64_t d, int64_t in_stride) {
  constexpr int VE = V16<T>::n;
  const int64_t per_row = d / VE, n = rows * per_row;
  for (int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; idx < n; idx += (int64_t)gridDim.x * blockDim.x) {
    const int64_t r = idx / per_row, i = (idx - r * per_row) * VE;
    const Vec<T, VE> g = ldvec<T, VE>(gate + r * in_stride + i), u = ldvec<T, VE>(up + r * in_stride + i);
    Vec<T, VE> o;
#pragma unroll
    for (int j = 0; j < VE; ++j) o.v[j] = from_f32<T>(gelu_tanh_f(to_f32(g.v[j])) * to_f32(u.v[j]));
    stvec<T, VE>(out + r * d + i, o);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void gelu_tanh_and_mul_kernel(T* __restrict__ out, const T* __restrict__ gate, const T* __restrict__ up,
                                                               int64_t rows, int64_t d, int64_t in_stride) {
  const int64_t n = rows * d;
  for (int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; idx < n; idx += (int64_t)gridDim.x * blockDim.x) {
    const int64_t r = idx / d, i = idx - r * d;
    out[idx] = from_f32<T>(gelu_tanh_f(to_f32(gate[r * in_stride + i])) * to_f32(up[r * in_stride + i]));
  }
}

// x[t][i] += sigmoid(g1[t][i] + b1[i]) * y1[t][i] (+ the same with g2, b2, y2 when y2 is given)
template <typename T>
__global__ __launch_bounds__(256) void gated_residual_kernel(
    float* __restrict__ x, const T* __restrict__ g1, const T* __restrict__ b1, const T* __restrict__ y1, const T* __restrict__ g2,
    const T* __restrict__ b2, const T* __restrict__ y2, int64_t rows, int64_t d, int64_t g_stride, int64_t y1_stride,
    int64_t y2_stride) {
  const int64_t n = rows * d;
  for (int64_t idx = (int64_t)blockIdx.x * blockDim.x + threadIdx.x; idx < n; idx += (int64_t)gridDim.x * blockDim.x) {
    const int64_t r = idx / d, i = idx - r * d;
    float add = sigmoid_f(to_f32(g1[r * g_stride + i]) + to_f32(b1[i])) * to_f32(y1[r * y1_stride + i]);
    if (y2 != nullptr) add += sigmoid_f(to_f32(g2[r * g_stride + i]) + to_f32(b2[i])) * to_f32(y2[r * y2_stride + i]);
    x[idx] += add;
  }
}

}  // namespace
}  // namespace mi355

using namespace mi355;

int mi355_layernorm_shift(void* h_out, void* hs_out, float* h_last, const float* x, const void* weight, const void* shift,
                          const float* state, const int32_t* req_to_state, const int64_t* req_pool_indices,
                          const int32_t* tok_req, const int32_t* seg_start, const int32_t* seg_len, const int64_t* positions,
                          int64_t tokens, int64_t hidden, float eps, int dtype, void* stream) {
  MI355_REQUIRE(h_out && x && weight, MI355_ERR_INVALID, "layernorm_shift: null pointer");
  MI355_REQUIRE(tokens >= 0 && hidden > 0 && hidden <= 16384, MI355_ERR_INVALID, "layernorm_shift: bad shape");
  MI355_REQUIRE(shift == nullptr || (hs_out && state && req_to_state && req_pool_indices && positions), MI355_ERR_INVALID,
                "layernorm_shift: the token shift needs hs_out, the state rows, the slot map and positions");
  MI355_REQUIRE((tok_req == nullptr) == (seg_start == nullptr) && (tok_req == nullptr) == (seg_len == nullptr), MI355_ERR_INVALID,
                "layernorm_shift: tok_req, seg_start and seg_len come together");
  if (tokens == 0) return MI355_OK;
  const size_t lds = (size_t)hidden * 2 * sizeof(float);
  MI355_DISPATCH_DTYPE(dtype, "layernorm_shift", {
    const bool wide = hidden % 4 == 0 && aligned16(x) && aligned16(h_out) && (!hs_out || aligned16(hs_out)) &&
                      (!state || aligned16(state));
    auto kern = wide ? layernorm_shift_kernel<T, 4> : layernorm_shift_kernel<T, 1>;
    if (lds > 48 * 1024) (void)hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(kern, dim3((unsigned)tokens), dim3(256), lds, (hipStream_t)stream, (T*)h_out, (T*)hs_out, h_last, x,
                       (const T*)weight, (const T*)shift, state, req_to_state, req_pool_indices, tok_req, seg_start, seg_len,
                       positions, hidden, eps);
  });
  MI355_CHECK_LAUNCH("layernorm_shift");
  return MI355_OK;
}

int mi355_bigram_embedding(float* x, const int64_t* ids, const void* table, const void* bigram, const int32_t* prev_token,
                           const int32_t* req_to_state, const int64_t* req_pool_indices, const int32_t* tok_req,
                           const int32_t* seg_start, const int32_t* seg_len, const int64_t* positions, int64_t tokens,
                           int64_t hidden, int64_t vocab, float scale, int64_t mul_prev, int64_t mul_cur, int64_t buckets,
                           int dtype, void* stream) {
  MI355_REQUIRE(x && ids && table && bigram && prev_token && req_to_state && req_pool_indices && positions, MI355_ERR_INVALID,
                "bigram_embedding: null pointer");
  MI355_REQUIRE(tokens >= 0 && hidden > 0 && vocab > 0 && buckets > 0, MI355_ERR_INVALID, "bigram_embedding: bad shape");
  MI355_REQUIRE((tok_req == nullptr) == (seg_start == nullptr) && (tok_req == nullptr) == (seg_len == nullptr), MI355_ERR_INVALID,
                "bigram_embedding: tok_req, seg_start and seg_len come together");
  if (tokens == 0) return MI355_OK;
  MI355_DISPATCH_DTYPE(dtype, "bigram_embedding", {
    hipLaunchKernelGGL((bigram_embedding_kernel<T>), dim3((unsigned)tokens), dim3(256), 0, (hipStream_t)stream, x, ids,
                       (const T*)table, (const T*)bigram, prev_token, req_to_state, req_pool_indices, tok_req, seg_start, seg_len,
                       positions, hidden, vocab, scale, mul_prev, mul_cur, buckets);
  });
  MI355_CHECK_LAUNCH("bigram_embedding");
  return MI355_OK;
}

int mi355_commit_sequence_state(float* state, int32_t* prev_token, const float* h_last, const int64_t* ids,
                                const int32_t* req_to_state, const int64_t* req_pool_indices, const int32_t* seg_start,
                                const int32_t* seg_len, int64_t batch, int64_t layers, int64_t hidden, int64_t state_layer_stride,
                                void* stream) {
  MI355_REQUIRE(state && h_last && ids && req_to_state && req_pool_indices, MI355_ERR_INVALID, "commit_sequence_state: null pointer");
  MI355_REQUIRE(batch >= 0 && layers > 0 && layers < 65536 && hidden > 0, MI355_ERR_INVALID, "commit_sequence_state: bad shape");
  MI355_REQUIRE((seg_start == nullptr) == (seg_len == nullptr), MI355_ERR_INVALID, "commit_sequence_state: seg_start and seg_len come together");
  if (batch == 0) return MI355_OK;
  hipLaunchKernelGGL(commit_state_kernel, dim3((unsigned)batch, (unsigned)layers), dim3(256), 0, (hipStream_t)stream, state,
                     prev_token, h_last, ids, req_to_state, req_pool_indices, seg_start, seg_len, batch, hidden, state_layer_stride);
  MI355_CHECK_LAUNCH("commit_sequence_state");
  return MI355_OK;
}

int mi355_gelu_tanh_and_mul(void* out, const void* gate, const void* up, int64_t rows, int64_t d, int64_t in_stride, int dtype,
                            void* stream) {
  MI355_REQUIRE(out && gate && up, MI355_ERR_INVALID, "gelu_tanh_and_mul: null pointer");
  MI355_REQUIRE(rows >= 0 && d > 0 && in_stride >= d, MI355_ERR_INVALID, "gelu_tanh_and_mul: bad shape");
  if (rows == 0) return MI355_OK;
  const int grid = (int)std::min<int64_t>((rows * d + 255) / 256, 256 * 16);
  MI355_DISPATCH_DTYPE(dtype, "gelu_tanh_and_mul", {
    constexpr int VE = V16<T>::n;
    if (d % VE == 0 && in_stride % VE == 0 && aligned16(out) && aligned16(gate) && aligned16(up)) {
      const int vgrid = (int)std::min<int64_t>((rows * (d / VE) + 255) / 256, 256 * 16);
      hipLaunchKernelGGL((gelu_tanh_and_mul_vec_kernel<T>), dim3(vgrid), dim3(256), 0, (hipStream_t)stream, (T*)out, (const T*)gate,
                         (const T*)up, rows, d, in_stride);
    } else {
      hipLaunchKernelGGL((gelu_tanh_and_mul_kernel<T>), dim3(grid), dim3(256), 0, (hipStream_t)stream, (T*)out, (const T*)gate,
                         (const T*)up, rows, d, in_stride);
    }
  });
  MI355_CHECK_LAUNCH("gelu_tanh_and_mul");
  return MI355_OK;
}

int mi355_gated_residual_add(float* x, const void* g1, const void* b1, const void* y1, const void* g2, const void* b2,
                             const void* y2, int64_t rows, int64_t d, int64_t g_stride, int64_t y1_stride, int64_t y2_stride,
                             int dtype, void* stream) {
  MI355_REQUIRE(x && g1 && b1 && y1, MI355_ERR_INVALID, "gated_residual_add: null pointer");
  MI355_REQUIRE(y2 == nullptr || (g2 && b2), MI355_ERR_INVALID, "gated_residual_add: the second branch needs its gate and bias");
  MI355_REQUIRE(rows >= 0 && d > 0, MI355_ERR_INVALID, "gated_residual_add: bad shape");
  if (rows == 0) return MI355_OK;
  const int grid = (int)std::min<int64_t>((rows * d + 255) / 256, 256 * 16);
  MI355_DISPATCH_DTYPE(dtype, "gated_residual_add", {
    hipLaunchKernelGGL((gated_residual_kernel<T>), dim3(grid), dim3(256), 0, (hipStream_t)stream, x, (const T*)g1, (const T*)b1,
                       (const T*)y1, (const T*)g2, (const T*)b2, (const T*)y2, rows, d, g_stride, y1_stride, y2_stride);
  });
  MI355_CHECK_LAUNCH("gated_residual_add");
  return MI355_OK;
}

static int norm_residual_add(LnAddParams& p, int64_t tokens, int rms, int dtype, void* stream) {
  const int64_t hidden = p.D;
  MI355_REQUIRE(p.x && p.y && p.w_out && (p.h != nullptr || p.w_next == nullptr), MI355_ERR_INVALID, "norm_residual_add: null pointer");
  MI355_REQUIRE((p.y2 == nullptr) == (p.gate == nullptr) && (p.rows == nullptr || p.n_rows > 0) && (p.coef == nullptr || p.rows != nullptr),
                MI355_ERR_INVALID, "norm_residual_add: the second branch comes with its gate, picked rows with their count, factors with rows");
  MI355_REQUIRE(tokens >= 0 && tokens < (1ll << 31) && hidden > 0 && hidden <= 32768 && p.y_stride >= hidden &&
                    (p.y2 == nullptr || p.y2_stride >= hidden), MI355_ERR_INVALID, "norm_residual_add: bad shape");
  if (tokens == 0) return MI355_OK;
  const bool vec = hidden % 8 == 0 && hidden <= 8192 && p.y_stride % 8 == 0 && aligned16(p.x) && aligned16(p.y) && aligned16(p.w_out) &&
                   (p.h == nullptr || aligned16(p.h)) && (p.w_next == nullptr || aligned16(p.w_next)) &&
                   (p.y2 == nullptr || (aligned16(p.y2) && p.y2_stride % 8 == 0));
  const dim3 grid((unsigned)tokens), block(256);
  const int keep = !vec ? 0 : hidden <= 2048 ? 1 : hidden <= 4096 ? 2 : 4;
  const size_t lds = keep == 0 ? (size_t)hidden * sizeof(float) : 0;
  MI355_DISPATCH_DTYPE(dtype, "norm_residual_add", {
    auto go = [&](auto kern) {
      if (lds > 48 * 1024) (void)hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      hipLaunchKernelGGL(kern, grid, block, lds, (hipStream_t)stream, p);
    };
    switch (keep) {
      case 1: go(rms ? layernorm_residual_add_kernel<T, 1, true> : layernorm_residual_add_kernel<T, 1, false>); break;
      case 2: go(rms ? layernorm_residual_add_kernel<T, 2, true> : layernorm_residual_add_kernel<T, 2, false>); break;
      case 4: go(rms ? layernorm_residual_add_kernel<T, 4, true> : layernorm_residual_add_kernel<T, 4, false>); break;
      default: go(rms ? layernorm_residual_add_kernel<T, 0, true> : layernorm_residual_add_kernel<T, 0, false>); break;
    }
  });
  MI355_CHECK_LAUNCH("norm_residual_add");
  return MI355_OK;
}

int mi355_layernorm_residual_add(float* x, void* h, const void* y, int64_t y_stride, const int32_t* rows, int n_rows, const void* y2,
                                 int64_t y2_stride, const float* y2_gate, int64_t gate_stride, const void* w_out, const void* w_next,
                                 int64_t tokens, int64_t hidden, float eps, int dtype, void* stream) {
  MI355_REQUIRE((h == nullptr) == (w_next == nullptr), MI355_ERR_INVALID, "layernorm_residual_add: the next norm comes with its result");
  LnAddParams p;
  p.x = x; p.h = h; p.y = y; p.rows = rows; p.coef = nullptr; p.y2 = y2; p.gate = y2_gate; p.w_out = w_out; p.w_next = w_next;
  p.y_stride = y_stride; p.y2_stride = y2_stride; p.gate_stride = gate_stride; p.D = hidden; p.n_rows = n_rows; p.eps = eps;
  return norm_residual_add(p, tokens, 0, dtype, stream);
}

int mi355_rmsnorm_residual_add_next(float* x, void* h, const void* y, int64_t y_stride, const int32_t* rows, const float* coef, int n_rows,
                                    const void* w_out, const void* w_next, int64_t tokens, int64_t hidden, float eps, int dtype,
                                    void* stream) {
  LnAddParams p;
  p.x = x; p.h = h; p.y = y; p.rows = rows; p.coef = coef; p.y2 = nullptr; p.gate = nullptr; p.w_out = w_out; p.w_next = w_next;
  p.y_stride = y_stride; p.y2_stride = 0; p.gate_stride = 0; p.D = hidden; p.n_rows = n_rows; p.eps = eps;
  return norm_residual_add(p, tokens, 1, dtype, stream);
}

int mi355_pass_entry(float* x, void* h, const void* y, int64_t y_stride, const float* table, const int64_t* ids, int64_t vocab,
                     const float* step, const void* w_next, int64_t tokens, int64_t hidden, float eps, int dtype, void* stream) {
  MI355_REQUIRE(x && h && y && table && ids && step && w_next, MI355_ERR_INVALID, "pass_entry: null pointer");
  MI355_REQUIRE(tokens >= 0 && tokens < (1ll << 31) && hidden > 0 && hidden <= 32768 && y_stride >= hidden && vocab > 0, MI355_ERR_INVALID,
                "pass_entry: bad shape");
  if (tokens == 0) return MI355_OK;
  PassEntryParams p;
  p.x = x; p.h = h; p.y = y; p.table = table; p.ids = ids; p.step = step; p.w_next = w_next; p.y_stride = y_stride; p.D = hidden;
  p.vocab = vocab; p.eps = eps;
  const bool vec = hidden % 8 == 0 && hidden <= 8192 && y_stride % 8 == 0 && aligned16(x) && aligned16(y) && aligned16(h) && aligned16(table) &&
                   aligned16(step) && aligned16(w_next);
  const int keep = !vec ? 0 : hidden <= 2048 ? 1 : hidden <= 4096 ? 2 : 4;
  const size_t lds = keep == 0 ? (size_t)hidden * sizeof(float) : 0;
  MI355_DISPATCH_DTYPE(dtype, "pass_entry", {
    auto kern = keep == 1 ? pass_entry_kernel<T, 1> : keep == 2 ? pass_entry_kernel<T, 2> : keep == 4 ? pass_entry_kernel<T, 4> : pass_entry_kernel<T, 0>;
    if (lds > 48 * 1024) (void)hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(kern, dim3((unsigned)tokens), dim3(256), lds, (hipStream_t)stream, p);
  });
  MI355_CHECK_LAUNCH("pass_entry");
  return MI355_OK;
}
