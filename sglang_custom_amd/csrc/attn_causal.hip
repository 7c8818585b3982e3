// Causal softmax attention over every earlier token, grouped key heads, per-layer key / value buffers [slots, G, maps * d] /
// [slots, G, dv] reached through the request table, with one or two score maps per head over the same values:
//     s_m[j] = (q[t, h, m] . K[j, g, m]) * scale,   cap > 0: s <- cap * tanh(s / cap),   for keys j <= pos(t),   g = h / (H / G)
//     a_m    = sum_j softmax(s_m)_j V[j, g]
//     one map:   out[t, h] = a_1
//     two maps:  o = a_1 - lambda * a_2;   out[t, h] = o / sqrt(mean(o^2) + eps) * out_scale
// times a gate per head (sigmoid of one logit) or per feature, if there is one.  Scores, weights and sums are fp32; in 16-bit
// runs the weights are rounded to the activation dtype as the second product's operand.
//
// Three kernels share the epilogue's arithmetic:
//   * causal_attention_tile_kernel    16-bit prompts and portions of prompts on 32x32x16 matrix cores.  A workgroup takes a run of
//     consecutive tokens of one sequence and the query heads of one key head: 128 (token, head) rows with one map, four waves of
//     32; with two maps 64 rows, waves 0 and 1 on the first map and 2 and 3 on the second, over the same V tile.
//   * causal_attention_token_kernel   16-bit single tokens (decode steps, single tokens inside a mixed batch) on 16x16x32 matrix
//     cores: the query heads of one key head are the columns of a tile, every wave walks key tiles of its own, keys travel from
//     global memory straight into matrix fragments.  A token's keys may be cut into ranges that a second launch merges.
//   * causal_attention_valu_kernel    everything else (fp32, widths without 16-byte rows): vector ALU, all fp32.
#include "common.cuh"

#include <algorithm>
#include <type_traits>

namespace mi355 {
namespace {

constexpr float CA_NEG = -1.0e30f;
constexpr float CA_LOG2E = 1.4426950408889634f;

struct CaArgs {
  void* out;
  const void* q;
  const void* k_cache;
  const void* v_cache;
  const int32_t* req_to_token;
  const int64_t* req_pool_indices;
  const int32_t* tok_req;
  const int64_t* positions;
  const int32_t* runs;     // [run][2] = first token, count; null: one token per run, run r = token r
  const void* gate;        // logits, or null
  float* partial;          // num_splits > 1: [split][token][head][map][dv + 2] = unnormalised result | running max | running sum
  int64_t num_runs, q_token_stride, out_token_stride, gate_token_stride, req_to_token_stride, tokens;
  int heads, kv_heads, d, dv, gate_per_feature, num_splits, rows_heads;
  float scale, cap, lambda, out_scale, eps;
};

__device__ __forceinline__ float ca_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
// sigmoid on the fast exponential, for 16-bit results
__device__ __forceinline__ float ca_sigmoid_fast(float z) {
  return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-CA_LOG2E * z));
}
// c * tanh(s / c) = c - 2 c / (e^(2 s / c) + 1): two transcendentals; k2 = 2 log2(e) / c.  The exponential's overflow gives c, its
// underflow -c.
__device__ __forceinline__ float ca_cap_fast(float s, float c, float k2) {
  return __builtin_fmaf(-2.0f * c, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(s * k2) + 1.0f), c);
}

// ------------------------------------------------------------------------------------------------ vector ALU
// 16 (token, head) rows per workgroup, key tiles of 32; lane (r = tid / 16, cx = tid % 16) owns row r's scores for keys cx and
// cx + 16 of a tile and its result columns cx, cx + 16, ...
// sm: Qs [16][maps d] | Ks [32][maps d + 1] | Vs [32][dv] | Ps [maps][16][32]
constexpr int CV_ROWS = 16;
constexpr int CV_KT = 32;

__device__ __forceinline__ float ca_row16_max(float x) {
#pragma unroll
  for (int o = 8; o > 0; o >>= 1) x = fmaxf(x, __shfl_xor(x, o, 16));
  return x;
}
__device__ __forceinline__ float ca_row16_sum(float x) {
#pragma unroll
  for (int o = 8; o > 0; o >>= 1) x += __shfl_xor(x, o, 16);
  return x;
}

template <typename T, int MAPS, int C>   // C: result columns per lane, dv <= 16 C
__global__ __launch_bounds__(256) void causal_attention_valu_kernel(CaArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int d = a.d, dv = a.dv, w = MAPS * d;
  float* Qs = sm;
  float* Ks = Qs + CV_ROWS * w;
  float* Vs = Ks + CV_KT * (w + 1);
  float* Ps = Vs + CV_KT * dv;
  __shared__ int row_pos[CV_ROWS];
  const int rep = a.heads / a.kv_heads, HR = a.rows_heads;
  const int chunks = (rep + HR - 1) / HR;
  const int g = blockIdx.y / chunks, hc = blockIdx.y - g * chunks;
  const int64_t bx = (int64_t)gridDim.x - 1 - blockIdx.x;
  const int64_t t0 = a.runs != nullptr ? a.runs[2 * bx] : bx;
  const int nt = a.runs != nullptr ? a.runs[2 * bx + 1] : 1;
  const int b = a.tok_req != nullptr ? a.tok_req[t0] : (int)t0;
  const int32_t* table = a.req_to_token + a.req_pool_indices[b] * a.req_to_token_stride;
  const int h0 = g * rep + hc * HR, nh = min(HR, rep - hc * HR);
  const int tid = threadIdx.x;
  const T* q = (const T*)a.q;
  const T* kc = (const T*)a.k_cache;
  const T* vc = (const T*)a.v_cache;
  for (int e = tid; e < CV_ROWS * w; e += 256) {
    const int r = e / w, i = e - r * w;
    const int tl = r / HR, hl = r - tl * HR;
    Qs[e] = (tl < nt && hl < nh) ? to_f32(q[(t0 + tl) * a.q_token_stride + (int64_t)(h0 + hl) * w + i]) : 0.f;
  }
  if (tid < CV_ROWS) {
    const int tl = tid / HR, hl = tid - tl * HR;
    row_pos[tid] = (tl < nt && hl < nh) ? (int)a.positions[t0 + tl] : -1;
  }
  const int last = (int)a.positions[t0] + nt - 1;       // the run's tokens are consecutive
  const int split = blockIdx.z;
  const int ntiles = last / CV_KT + 1;
  const int per = (ntiles + a.num_splits - 1) / a.num_splits;
  const int tile_lo = split * per, tile_hi = min(ntiles, tile_lo + per);
  const int r = tid >> 4, cx = tid & 15;
  float run_m[MAPS], run_l[MAPS], acc[MAPS][C];
#pragma unroll
  for (int m = 0; m < MAPS; ++m) {
    run_m[m] = CA_NEG;
    run_l[m] = 0.f;
#pragma unroll
    for (int c = 0; c < C; ++c) acc[m][c] = 0.f;
  }
  for (int tile = tile_lo; tile < tile_hi; ++tile) {
    const int j0 = tile * CV_KT;
    __syncthreads();
    for (int e = tid; e < CV_KT * w; e += 256) {
      const int kk = e / w, i = e - kk * w;
      Ks[kk * (w + 1) + i] = j0 + kk <= last ? to_f32(kc[((int64_t)table[j0 + kk] * a.kv_heads + g) * w + i]) : 0.f;
    }
    for (int e = tid; e < CV_KT * dv; e += 256) {
      const int kk = e / dv, i = e - kk * dv;
      Vs[e] = j0 + kk <= last ? to_f32(vc[((int64_t)table[j0 + kk] * a.kv_heads + g) * dv + i]) : 0.f;
    }
    __syncthreads();
    const int rp = row_pos[r];
    float alpha[MAPS];
#pragma unroll
    for (int m = 0; m < MAPS; ++m) {
      float sc[CV_KT / 16], tmax = CA_NEG;
#pragma unroll
      for (int u = 0; u < CV_KT / 16; ++u) {
        const int kk = cx + 16 * u;
        float s = 0.f;
        for (int i = 0; i < d; ++i) s = fmaf(Qs[r * w + m * d + i], Ks[kk * (w + 1) + m * d + i], s);
        s *= a.scale;
        if (a.cap > 0.f) s = a.cap * tanhf(s / a.cap);
        sc[u] = j0 + kk <= rp ? s : CA_NEG;
        tmax = fmaxf(tmax, sc[u]);
      }
      const float new_m = fmaxf(run_m[m], ca_row16_max(tmax));
      alpha[m] = expf(run_m[m] - new_m);              // 1 when nothing changed, also for rows that have seen nothing yet
      float psum = 0.f;
#pragma unroll
      for (int u = 0; u < CV_KT / 16; ++u) {
        const float p = j0 + cx + 16 * u <= rp ? expf(sc[u] - new_m) : 0.f;
        Ps[(m * CV_ROWS + r) * CV_KT + cx + 16 * u] = p;
        psum += p;
      }
      run_l[m] = run_l[m] * alpha[m] + ca_row16_sum(psum);
      run_m[m] = new_m;
    }
    __syncthreads();
#pragma unroll
    for (int m = 0; m < MAPS; ++m)
#pragma unroll
      for (int c = 0; c < C; ++c) acc[m][c] *= alpha[m];
    for (int kk = 0; kk < CV_KT; ++kk) {
#pragma unroll
      for (int c = 0; c < C; ++c) {
        const int col = cx + 16 * c;
        if (col < dv) {
          const float v = Vs[kk * dv + col];
#pragma unroll
          for (int m = 0; m < MAPS; ++m) acc[m][c] = fmaf(Ps[(m * CV_ROWS + r) * CV_KT + kk], v, acc[m][c]);
        }
      }
    }
  }
  const int tl = r / HR, hl = r - tl * HR;
  const bool live = tl < nt && hl < nh;
  const int64_t t = t0 + tl;
  const int h = h0 + hl;
  if (a.num_splits > 1) {
    if (!live) return;
#pragma unroll
    for (int m = 0; m < MAPS; ++m) {
      float* part = a.partial + ((((int64_t)split * a.tokens + t) * a.heads + h) * MAPS + m) * (dv + 2);
#pragma unroll
      for (int c = 0; c < C; ++c)
        if (cx + 16 * c < dv) part[cx + 16 * c] = acc[m][c];
      if (cx == 0) { part[dv] = run_m[m]; part[dv + 1] = run_l[m]; }
    }
    return;
  }
  float o[C], q2 = 0.f;
  const float inv1 = run_l[0] > 0.f ? 1.0f / run_l[0] : 0.f;
  float inv2 = 0.f;
  if constexpr (MAPS == 2) inv2 = run_l[1] > 0.f ? a.lambda / run_l[1] : 0.f;
#pragma unroll
  for (int c = 0; c < C; ++c) {
    o[c] = cx + 16 * c < dv ? acc[0][c] * inv1 : 0.f;
    if constexpr (MAPS == 2) o[c] -= cx + 16 * c < dv ? acc[1][c] * inv2 : 0.f;
    q2 += o[c] * o[c];
  }
  float mul = 1.f;
  if constexpr (MAPS == 2) mul = a.out_scale / sqrtf(ca_row16_sum(q2) / (float)dv + a.eps);
  if (!live) return;
  const T* gt = (const T*)a.gate + t * a.gate_token_stride;
  if (a.gate != nullptr && !a.gate_per_feature) mul *= ca_sigmoid(to_f32(gt[h]));
#pragma unroll
  for (int c = 0; c < C; ++c) {
    const int col = cx + 16 * c;
    if (col >= dv) continue;
    float y = o[c] * mul;
    if (a.gate != nullptr && a.gate_per_feature) y *= ca_sigmoid(to_f32(gt[(int64_t)h * dv + col]));
    ((T*)a.out)[t * a.out_token_stride + (int64_t)h * dv + col] = from_f32<T>(y);
  }
}

// Ranges of a token's keys, in order: a_m = sum_s acc_s e^(m_s - M) / sum_s l_s e^(m_s - M), M = max_s m_s; then the epilogue.
// One wave per (token, head); a lane owns up to 8 columns lane, lane + 64, ... (dv <= 512).
template <typename T, int MAPS>
__global__ __launch_bounds__(256) void causal_attention_merge_kernel(CaArgs a) {
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  const int64_t idx = (int64_t)blockIdx.x * 4 + wv;
  if (idx >= a.num_runs * a.heads) return;
  const int64_t run = idx / a.heads;
  const int h = (int)(idx - run * a.heads);
  const int64_t t = a.runs != nullptr ? a.runs[2 * run] : run;
  const int dv = a.dv;
  const int64_t stride = a.tokens * a.heads * MAPS * (int64_t)(dv + 2);
  float o[8];
#pragma unroll
  for (int u = 0; u < 8; ++u) o[u] = 0.f;
#pragma unroll
  for (int m = 0; m < MAPS; ++m) {
    const float* p0 = a.partial + ((t * a.heads + h) * MAPS + m) * (int64_t)(dv + 2);
    // lane s holds range s (at most 64 of them)
    const bool has = lane < a.num_splits;
    const float ms = has ? p0[lane * stride + dv] : CA_NEG, ls = has ? p0[lane * stride + dv + 1] : 0.f;
    const float w = expf(ms - wave_max(ms));
    const float L = wave_sum(ls * w);
    const float wn = w * (m == 1 ? -a.lambda : 1.0f) * (L > 0.f ? 1.0f / L : 0.f);
#pragma unroll 4
    for (int s = 0; s < a.num_splits; ++s) {
      const float f = __shfl(wn, s, 64);
#pragma unroll
      for (int u = 0; u < 8; ++u)
        if (64 * u < dv && lane + 64 * u < dv) o[u] += p0[s * stride + lane + 64 * u] * f;
    }
  }
  float mul = 1.f;
  if constexpr (MAPS == 2) {
    float q2 = 0.f;
#pragma unroll
    for (int u = 0; u < 8; ++u) q2 += o[u] * o[u];
    mul = a.out_scale / sqrtf(wave_sum(q2) / (float)dv + a.eps);
  }
  const T* gt = (const T*)a.gate + t * a.gate_token_stride;
  if (a.gate != nullptr && !a.gate_per_feature) mul *= ca_sigmoid(to_f32(gt[h]));
#pragma unroll
  for (int u = 0; u < 8; ++u) {
    const int col = lane + 64 * u;
    if (col >= dv) continue;
    float y = o[u] * mul;
    if (a.gate != nullptr && a.gate_per_feature) y *= ca_sigmoid(to_f32(gt[(int64_t)h * dv + col]));
    ((T*)a.out)[t * a.out_token_stride + (int64_t)h * dv + col] = from_f32<T>(y);
  }
}

// ------------------------------------------------------------------------------------------------ prompts, matrix cores
// S^T = K Q^T (A = 32 key rows from LDS, B = the wave's 32 queries in registers), so a lane owns its query's scores, and the
// rounded weights are the B operand of O^T += V^T P^T (A by transposed reads of the row-major V tile); see the layout notes of
// the 32x32x16 instruction in common.cuh.  Key tiles of 64 (32 where results and queries fill the registers), the next tile in
// registers and the cache slots of the one after it while the current one is multiplied.
// LDS rows: K rows have an odd number of 16-byte chunks (16 consecutive rows start in 16 different bank groups), V rows a number
// that is 4 or 12 modulo 16 (the four rows of a transposed read start 64 bytes apart).
// KS: score steps of 16 features (d <= 16 KS, the rest zero), VT: 32-column tiles of the result (dv <= 32 VT).
template <int KS, int MAPS> constexpr int ca_k_pitch() { return (2 * KS * MAPS + 1) * 16; }
template <int VT> constexpr int ca_v_pitch() { return 4 * (VT | 1) * 16; }
// keys per tile, and workgroups per CU: two where queries, results and the staged tile leave room in 256 registers
constexpr int ca_regs(int ks, int vt, int maps, int keys) { return 4 * ks + 16 * vt + keys * (2 * ks * maps + 4 * vt) / 64 + keys / 2; }
constexpr int ca_keys(int ks, int vt, int maps) { return ca_regs(ks, vt, maps, 64) <= 176 || ca_regs(ks, vt, maps, 32) > 208 ? 64 : 32; }
constexpr int ca_waves(int ks, int vt, int maps) { return ca_regs(ks, vt, maps, ca_keys(ks, vt, maps)) <= 208 ? 2 : 1; }
template <int KS, int VT, int MAPS> constexpr size_t ca_tile_lds() {
  const size_t kv = (size_t)ca_keys(KS, VT, MAPS) * (ca_k_pitch<KS, MAPS>() + ca_v_pitch<VT>());
  const size_t ex = MAPS == 2 ? (size_t)64 * (32 * VT + 4) * 4 : 0;
  return kv > ex ? kv : ex;
}

template <typename T, int KS, int VT, int MAPS, bool CAP>
__device__ __forceinline__ void causal_attention_tile_body(const CaArgs& a, char* sm) {
  using frag = typename Mfma32<T>::frag;
  constexpr int KP = ca_k_pitch<KS, MAPS>(), VP = ca_v_pitch<VT>();
  constexpr int BN = ca_keys(KS, VT, MAPS), HF = BN / 32;      // keys per tile, in halves of 32
  constexpr int KL = 2 * KS * MAPS, VL = 4 * VT;               // 16-byte chunks of a (padded) key and value row
  constexpr int KN = BN * KL / 256, VN = BN * VL / 256;        // chunks per thread
  static_assert(KN >= 1 && VN >= 1 && 256 % KL == 0 && 256 % VL == 0, "a thread's chunks lie in one column");
  char* ks = sm;
  char* vs = sm + BN * KP;
  const int rep = a.heads / a.kv_heads, HR = a.rows_heads;
  const int chunks = (rep + HR - 1) / HR, per_run = a.kv_heads * chunks;
  // consecutive workgroups differ in the key head (they go round-robin over the XCDs); long, late runs first
  const int64_t run = a.num_runs - 1 - blockIdx.x / per_run;
  const int y = blockIdx.x % per_run, g = y / chunks, hc = y - g * chunks;
  const int64_t t0 = a.runs[2 * run];
  const int nt = a.runs[2 * run + 1];
  const int b = a.tok_req[t0];
  const int32_t* table = a.req_to_token + a.req_pool_indices[b] * a.req_to_token_stride;
  const int h0 = g * rep + hc * HR, nh = min(HR, rep - hc * HR);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int j32 = lane & 31, hh = lane >> 5;
  const int map = MAPS == 2 ? wave >> 1 : 0, qw = MAPS == 2 ? wave & 1 : wave;     // this wave's map and block of 32 rows
  const int d = a.d, dv = a.dv;
  const int first = (int)a.positions[t0], last = first + nt - 1;
  const int row = 32 * qw + j32;
  const int tl = row / HR, hl = row - tl * HR;
  const bool live = tl < nt && hl < nh;
  const int tl_c = min(tl, nt - 1), h = h0 + min(hl, nh - 1);
  const int my_limit = first + tl_c;                                               // last key this lane's query sees
  const int wave_min_limit = first + min(32 * qw / HR, nt - 1), wave_max_limit = first + min((32 * qw + 31) / HR, nt - 1);
  const bool wave_idle = 32 * qw / HR >= nt;                                       // no live row in this wave

  frag qf[KS];
  {
    const T* qp = (const T*)a.q + (t0 + tl_c) * a.q_token_stride + ((int64_t)h * MAPS + map) * d;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int i = 16 * s + 8 * hh;
      const frag zero = {};
      const frag v = *reinterpret_cast<const frag*>(qp + min(i, d - 8));
      qf[s] = i < d ? v : zero;
    }
  }
  // staging: a thread owns one chunk column of the K rows tid / KL + u * 256 / KL and of the V rows tid / VL + u * 256 / VL; a map's
  // features past d are zeros in the K tile (the queries' are too, but 0 * garbage may be NaN), columns past dv are left alone
  const int kr0 = threadIdx.x / KL, kch = threadIdx.x % KL, kmap = kch / (2 * KS), kc0 = (kch % (2 * KS)) * 8;
  const int vr0 = threadIdx.x / VL, vc0 = (threadIdx.x % VL) * 8;
  const bool klive = kc0 < d, vlive = vc0 < dv;
  const T* kc = (const T*)a.k_cache + ((int64_t)g * MAPS + kmap) * d + (klive ? kc0 : 0);
  const T* vc = (const T*)a.v_cache + (int64_t)g * dv + (vlive ? vc0 : 0);
  const int64_t krow = (int64_t)a.kv_heads * MAPS * d, vrow_ = (int64_t)a.kv_heads * dv;
  char* kst = ks + kr0 * KP + 16 * kch;
  char* vst = vs + vr0 * VP + 2 * vc0;
  int kslot[KN], vslot[KL == VL ? 1 : VN];
  Vec<T, 8> kreg[KN], vreg[VN];
  auto load_slots = [&](int kt) {         // keys past the last one are clamped (and masked below)
#pragma unroll
    for (int u = 0; u < KN; ++u) kslot[u] = table[min(kt * BN + kr0 + u * (256 / KL), last)];
    if constexpr (KL != VL) {
#pragma unroll
      for (int u = 0; u < VN; ++u) vslot[u] = table[min(kt * BN + vr0 + u * (256 / VL), last)];
    }
  };
  auto load_tile = [&]() {
#pragma unroll
    for (int u = 0; u < KN; ++u) kreg[u] = ldvec<T, 8>(kc + (int64_t)kslot[u] * krow);
#pragma unroll
    for (int u = 0; u < VN; ++u) vreg[u] = ldvec<T, 8>(vc + (int64_t)(KL == VL ? kslot[u % KN] : vslot[KL == VL ? 0 : u]) * vrow_);
  };
  auto store_tile = [&]() {
    const Vec<T, 8> zero = __builtin_bit_cast(Vec<T, 8>, lds_u32x4{0, 0, 0, 0});
#pragma unroll
    for (int u = 0; u < KN; ++u) lds_store16(kst + u * (256 / KL) * KP, klive ? kreg[u] : zero);
    if (vlive) {
#pragma unroll
      for (int u = 0; u < VN; ++u) lds_store16(vst + u * (256 / VL) * VP, vreg[u]);
    }
  };

  f32x16 ot[VT];
#pragma unroll
  for (int c = 0; c < VT; ++c)
#pragma unroll
    for (int i = 0; i < 16; ++i) ot[c][i] = 0.f;
  float m = -INFINITY, lsum = 0.f;
  // scores enter the exponent as log2(e) times the (scaled, capped) score
  const float qmul = CAP ? CA_LOG2E : a.scale * CA_LOG2E;
  const float k2 = CAP ? 2.0f * CA_LOG2E * a.scale / a.cap : 0.f;
  const char* k_rd = ks + KP * j32 + 16 * (map * 2 * KS + hh);
  auto k_frag = [&](int s, int hf) -> frag { return lds_load16<frag>(k_rd + 32 * KP * hf + 32 * s); };
  const int l16 = lane & 15, dhalf = (lane >> 4) & 1, tq = l16 >> 2, tpp = l16 & 3;
  const char* v_rd = vs + VP * (4 * hh + tq) + 32 * dhalf + 8 * tpp;
  const int n_tiles = last / BN + 1;
  load_slots(0);
  load_tile();
  load_slots(min(1, n_tiles - 1));
  for (int kt = 0; kt < n_tiles; ++kt) {
    __syncthreads();            // the previous tile is consumed
    store_tile();
    __syncthreads();
    if (kt + 1 < n_tiles) {
      load_tile();
      load_slots(min(kt + 2, n_tiles - 1));
    }
    if (wave_idle || kt * BN > wave_max_limit) continue;      // nothing of this tile is seen by this wave (wave-uniform)
    f32x16 st[HF];
#pragma unroll
    for (int hf = 0; hf < HF; ++hf)
#pragma unroll
      for (int i = 0; i < 16; ++i) st[hf][i] = 0.f;
    // fragments are read two steps ahead of the products that use them
    frag kr[3][HF];
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int hf = 0; hf < HF; ++hf) kr[s][hf] = k_frag(s, hf);
    typename TrRead<T>::v4 vlo[4], vhi[4];                    // ring of four (16-key step, column tile) fragments
    auto v_read = [&](int i, int slot) {
      const int u = i / VT, c = i % VT;
      vlo[slot] = TrRead<T>::run(reinterpret_cast<const T*>(v_rd + VP * (16 * u) + 64 * c));
      vhi[slot] = TrRead<T>::run(reinterpret_cast<const T*>(v_rd + VP * (16 * u + 8) + 64 * c));
    };
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      if (s + 2 < KS) {
#pragma unroll
        for (int hf = 0; hf < HF; ++hf) kr[(s + 2) % 3][hf] = k_frag(s + 2, hf);
      } else if (s == KS - 2) {
        v_read(0, 0);
        v_read(1, 1);
      } else {
        v_read(2, 2);
        v_read(3, 3);
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int hf = 0; hf < HF; ++hf) st[hf] = Mfma32<T>::run(kr[s % 3][hf], qf[s], st[hf]);
      __builtin_amdgcn_sched_barrier(0);
    }
    if constexpr (CAP) {
#pragma unroll
      for (int hf = 0; hf < HF; ++hf)
#pragma unroll
        for (int i = 0; i < 16; ++i) st[hf][i] = ca_cap_fast(st[hf][i], a.cap, k2);
    }
    float mloc = -INFINITY;
    if (kt * BN + BN - 1 > wave_min_limit) {                      // only tiles that cross the wave's diagonal are masked
      const int lim = my_limit - kt * BN - 4 * hh;
#pragma unroll
      for (int hf = 0; hf < HF; ++hf)
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const float x = (32 * hf + 8 * (i >> 2) + (i & 3)) > lim ? -INFINITY : st[hf][i];
          st[hf][i] = x;
          mloc = fmaxf(mloc, x);
        }
    } else {
#pragma unroll
      for (int hf = 0; hf < HF; ++hf)
#pragma unroll
        for (int i = 0; i < 16; ++i) mloc = fmaxf(mloc, st[hf][i]);
    }
    mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
    const float mnew = fmaxf(m, mloc * qmul);
    const float ms = mnew == -INFINITY ? 0.f : mnew;
    const float alpha = __builtin_amdgcn_exp2f(m - ms);
    m = mnew;
    float psum = 0.f;
    frag pb[2 * HF];
#pragma unroll
    for (int hf = 0; hf < HF; ++hf)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const float pe = __builtin_amdgcn_exp2f(__builtin_fmaf(st[hf][i], qmul, -ms));
        psum += pe;
        pb[2 * hf + (i >> 3)][i & 7] = (T)pe;
      }
    lsum = lsum * alpha + psum;
    if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {
#pragma unroll
      for (int c = 0; c < VT; ++c) ot[c] *= alpha;
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int i = 0; i < 2 * HF * VT; ++i) {                        // fragment i + 4 is requested right behind product i
      frag va;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        va[e] = vlo[i & 3][e];
        va[4 + e] = vhi[i & 3][e];
      }
      ot[i % VT] = Mfma32<T>::run(va, pb[i / VT], ot[i % VT]);
      __builtin_amdgcn_sched_barrier(0);
      if (i + 4 < 2 * HF * VT) {
        v_read(i + 4, i & 3);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
  }
  lsum += __shfl_xor(lsum, 32, 64);
  const float inv = lsum > 0.f ? 1.f / lsum : 0.f;
  float mul = inv;
  if constexpr (MAPS == 2) {
    // the second map's waves hand lambda * a_2 to the first map's, row by row, through the tiles' memory
    constexpr int XP = 32 * VT + 4;
    float* ex = reinterpret_cast<float*>(sm);
    __syncthreads();
    if (map == 1) {
      const float f = inv * a.lambda;
#pragma unroll
      for (int c = 0; c < VT; ++c)
#pragma unroll
        for (int rq = 0; rq < 4; ++rq) {
          Vec<float, 4> w;
#pragma unroll
          for (int r = 0; r < 4; ++r) w.v[r] = ot[c][4 * rq + r] * f;
          lds_store16(ex + row * XP + 32 * c + 8 * rq + 4 * hh, w);
        }
    }
    __syncthreads();
    if (map == 1) return;
    float q2 = 0.f;
#pragma unroll
    for (int c = 0; c < VT; ++c)
#pragma unroll
      for (int rq = 0; rq < 4; ++rq) {
        const int col = 32 * c + 8 * rq + 4 * hh;
        const Vec<float, 4> w = lds_load16<Vec<float, 4>>(ex + row * XP + col);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float o = col < dv ? ot[c][4 * rq + r] * inv - w.v[r] : 0.f;
          ot[c][4 * rq + r] = o;
          q2 += o * o;
        }
      }
    q2 += __shfl_xor(q2, 32, 64);
    mul = a.out_scale / sqrtf(q2 / (float)dv + a.eps);
  }
  if (!live) return;
  const int64_t t = t0 + tl;
  const T* gt = (const T*)a.gate + t * a.gate_token_stride;
  if (a.gate != nullptr && !a.gate_per_feature) mul *= ca_sigmoid_fast(to_f32(gt[h]));
  T* op = (T*)a.out + t * a.out_token_stride + (int64_t)h * dv;
#pragma unroll
  for (int c = 0; c < VT; ++c)
#pragma unroll
    for (int rq = 0; rq < 4; ++rq) {
      const int col = 32 * c + 8 * rq + 4 * hh;
      if (col >= dv) continue;
      Vec<T, 4> w;
      if (a.gate != nullptr && a.gate_per_feature) {
        const Vec<T, 4> z = ldvec<T, 4>(gt + (int64_t)h * dv + col);
#pragma unroll
        for (int r = 0; r < 4; ++r) w.v[r] = from_f32<T>(ot[c][4 * rq + r] * mul * ca_sigmoid_fast(to_f32(z.v[r])));
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) w.v[r] = from_f32<T>(ot[c][4 * rq + r] * mul);
      }
      stvec<T, 4>(op + col, w);
    }
}

template <typename T, int KS, int VT, int MAPS, bool CAP>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(ca_waves(KS, VT, MAPS), ca_waves(KS, VT, MAPS))))
void causal_attention_tile_kernel(CaArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smt[];
  causal_attention_tile_body<T, KS, VT, MAPS, CAP>(a, smt);
}

// ------------------------------------------------------------------------------------------------ single tokens, matrix cores
// A workgroup: one token, one key head, up to 16 of its query heads, one range of the token's keys.  A wave takes key tiles (32 keys)
// of the range on its own: one map, every fourth tile; two maps, waves 0 and 2 the first map and 1 and 3 the second, every second
// tile (the pair's second reading of the values comes from L2).  S = K Q^T puts head l & 15 and keys 4 (l >> 4) + r of two 16-key
// halves into lane l; the rounded weights are the B operand of O^T += V^T P^T with the keys in just that order; V goes through a
// wave-private piece of LDS for the transposed reads.  The waves' results meet in LDS at the end.
// KS: score steps of 32 features (d <= 32 KS, the rest zero), VC: 16-column tiles of the result (dv <= 16 VC).
template <int VC> constexpr int ct_v_pitch() { return 4 * (((VC + 1) / 2) | 1) * 16; }
template <int VC> constexpr size_t ct_lds() {
  const size_t v = (size_t)4 * 32 * ct_v_pitch<VC>(), ex = (size_t)2 * 16 * (16 * VC + 4) * 4;
  return v > ex ? v : ex;
}

template <typename T, int KS, int VC, int MAPS>
__global__ __launch_bounds__(256) void causal_attention_token_kernel(CaArgs a) {
  extern __shared__ __attribute__((aligned(16))) char smd[];
  __shared__ float red_m[4][16], red_l[4][16];
  using frag = typename Mfma<T>::frag;
  constexpr int VP = ct_v_pitch<VC>();
  constexpr int VL = 2 * VC, VN = VC;         // 16-byte chunks of a (padded) value row; chunks of a V tile per lane
  constexpr int STREAMS = 4 / MAPS;           // waves that walk the range side by side
  const int rep = a.heads / a.kv_heads;
  const int chunks = (rep + 15) / 16, per_run = a.kv_heads * chunks;
  const int64_t run = blockIdx.x / per_run;
  const int y = blockIdx.x % per_run, g = y / chunks, hc = y - g * chunks;
  const int64_t t = a.runs != nullptr ? a.runs[2 * run] : run;
  const int b = a.tok_req != nullptr ? a.tok_req[t] : (int)t;
  const int32_t* table = a.req_to_token + a.req_pool_indices[b] * a.req_to_token_stride;
  const int h0 = g * rep + hc * 16, nh = min(16, rep - hc * 16);
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int map = MAPS == 2 ? wave & 1 : 0, stream = MAPS == 2 ? wave >> 1 : wave;
  const int li = lane & 15, lg = lane >> 4;
  const int d = a.d, dv = a.dv;
  const int len = (int)a.positions[t] + 1;
  // the token's own length is cut into ranges of whole tiles of 32, at least eight tiles each: short sequences fill fewer ranges
  const int ntiles = (len + 31) / 32;
  const int per = max((ntiles + a.num_splits - 1) / a.num_splits, a.num_splits > 1 ? min(8, ntiles) : 1);
  const int split = blockIdx.y;
  const int tile_lo = split * per, tile_hi = min(ntiles, tile_lo + per);
  const T* kc = (const T*)a.k_cache + ((int64_t)g * MAPS + map) * d;
  const int64_t krow = (int64_t)a.kv_heads * MAPS * d, vrow_ = (int64_t)a.kv_heads * dv;
  frag qf[KS];
  const frag zero = {};
  {
    const T* qp = (const T*)a.q + t * a.q_token_stride + ((int64_t)(h0 + min(li, nh - 1)) * MAPS + map) * d;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int i = 32 * s + 8 * lg;
      const frag v = *reinterpret_cast<const frag*>(qp + min(i, d - 8));
      qf[s] = i < d ? v : zero;
    }
  }
  f32x4 acc[VC];
  float run_m = -INFINITY, run_l = 0.f;
#pragma unroll
  for (int c = 0; c < VC; ++c) acc[c] = f32x4{0.f, 0.f, 0.f, 0.f};
  char* vsw = smd + wave * 32 * VP;
  // a lane owns one chunk column of the V rows lane / VL + u * 64 / VL; columns past dv are left alone
  const int vr0 = lane / VL, vc0 = (lane % VL) * 8;
  const bool vlive = vc0 < dv;
  const T* vc = (const T*)a.v_cache + (int64_t)g * dv + (vlive ? vc0 : 0);
  char* vst = vsw + vr0 * VP + 2 * vc0;
  const bool cap = a.cap > 0.f;
  const float qmul = cap ? CA_LOG2E : a.scale * CA_LOG2E;
  const float k2 = cap ? 2.0f * CA_LOG2E * a.scale / a.cap : 0.f;
  frag kf[2][KS];
  Vec<T, 8> vreg[VN];
  int slot = 0;                               // lane l & 31: the cache slot of key l & 31 of the tile whose rows come next
  auto load_slots = [&](int tile) { slot = table[min(tile * 32 + (lane & 31), len - 1)]; };
  auto load_rows = [&]() {
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      const T* kp = kc + (int64_t)__shfl(slot, 16 * hf + li, 64) * krow;
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int i = 32 * s + 8 * lg;
        const frag v = *reinterpret_cast<const frag*>(kp + min(i, d - 8));
        kf[hf][s] = i < d ? v : zero;
      }
    }
#pragma unroll
    for (int u = 0; u < VN; ++u) vreg[u] = ldvec<T, 8>(vc + (int64_t)__shfl(slot, vr0 + u * (64 / VL), 64) * vrow_);
  };
  const char* v_rd = vsw + VP * (4 * lg + (li >> 2)) + 8 * (li & 3);
  int tile = tile_lo + stream;
  if (tile < tile_hi) {                       // wave-uniform
    load_slots(tile);
    load_rows();
    load_slots(min(tile + STREAMS, ntiles - 1));
  }
  for (; tile < tile_hi; tile += STREAMS) {
    // V to LDS (this wave's piece; a wave's LDS accesses stay in order), scores from the K fragments
    if (vlive) {
#pragma unroll
      for (int u = 0; u < VN; ++u) lds_store16(vst + u * (64 / VL) * VP, vreg[u]);
    }
    f32x4 st[2];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      st[hf] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < KS; ++s) st[hf] = Mfma<T>::run(kf[hf][s], qf[s], st[hf]);
    }
    if (tile + STREAMS < tile_hi) {           // the next tile's rows are in flight during the rest
      load_rows();
      load_slots(min(tile + 2 * STREAMS, ntiles - 1));
    }
    const int lim = len - 1 - tile * 32 - 4 * lg;      // last visible key, relative to this lane's first
    float mloc = -INFINITY;
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float x = st[hf][r];
        if (cap) x = ca_cap_fast(x, a.cap, k2);
        x = 16 * hf + r > lim ? -INFINITY : x;
        st[hf][r] = x;
        mloc = fmaxf(mloc, x);
      }
    mloc = fmaxf(mloc, __shfl_xor(mloc, 16, 64));
    mloc = fmaxf(mloc, __shfl_xor(mloc, 32, 64));
    const float mnew = fmaxf(run_m, mloc * qmul);      // finite: a tile's first key is always visible
    const float alpha = __builtin_amdgcn_exp2f(run_m - mnew);
    run_m = mnew;
    float psum = 0.f;
    frag pb;
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float pe = __builtin_amdgcn_exp2f(__builtin_fmaf(st[hf][r], qmul, -mnew));
        psum += pe;
        pb[4 * hf + r] = (T)pe;
      }
    run_l = run_l * alpha + psum;             // this lane's keys alone; the lanes of a head are added at the end
    if (__builtin_amdgcn_ballot_w64(alpha != 1.f) != 0) {
#pragma unroll
      for (int c = 0; c < VC; ++c) acc[c] *= alpha;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int c = 0; c < VC; ++c) {
      typename TrRead<T>::v4 both[2];
      both[0] = TrRead<T>::run(reinterpret_cast<const T*>(v_rd + 32 * c));
      both[1] = TrRead<T>::run(reinterpret_cast<const T*>(v_rd + 16 * VP + 32 * c));
      acc[c] = Mfma<T>::run(__builtin_bit_cast(frag, both), pb, acc[c]);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  // ---- the streams of a map: common maximum, sums, then rounds of adding through LDS; waves 0 (and 1: the second map) keep the result
  run_l += __shfl_xor(run_l, 16, 64);
  run_l += __shfl_xor(run_l, 32, 64);
  if (lg == 0) { red_m[wave][li] = run_m; red_l[wave][li] = run_l; }
  __syncthreads();
  float M = -INFINITY, L = 0.f;
#pragma unroll
  for (int w = 0; w < STREAMS; ++w) M = fmaxf(M, red_m[w * MAPS + map][li]);
  const float Ms = M == -INFINITY ? 0.f : M;
#pragma unroll
  for (int w = 0; w < STREAMS; ++w) L += red_l[w * MAPS + map][li] * __builtin_amdgcn_exp2f(red_m[w * MAPS + map][li] - Ms);
  const float f = __builtin_amdgcn_exp2f(run_m - Ms);
#pragma unroll
  for (int c = 0; c < VC; ++c) acc[c] *= f;
  constexpr int XP = 16 * VC + 4;
  float* ex = reinterpret_cast<float*>(smd);
  auto hand = [&](int piece, float factor) {
#pragma unroll
    for (int c = 0; c < VC; ++c) lds_store16(ex + (piece * 16 + li) * XP + 16 * c + 4 * lg, __builtin_bit_cast(Vec<float, 4>, acc[c] * factor));
  };
  auto take = [&](int piece, float sign) {
#pragma unroll
    for (int c = 0; c < VC; ++c) acc[c] += lds_load16<f32x4>(ex + (piece * 16 + li) * XP + 16 * c + 4 * lg) * sign;
  };
#pragma unroll
  for (int step = 2; step >= MAPS; step >>= 1) {      // waves step .. 2 step - 1 onto waves 0 .. step - 1
    if (wave >= step && wave < 2 * step) hand(wave - step, 1.f);
    __syncthreads();
    if (wave < step) take(wave, 1.f);
    __syncthreads();
  }
  const int h = h0 + li;
  // lane: head li, columns 16 c + 4 lg + r
  if (a.num_splits > 1) {
    if (wave >= MAPS || li >= nh) return;
    float* part = a.partial + ((((int64_t)split * a.tokens + t) * a.heads + h) * MAPS + map) * (dv + 2);
#pragma unroll
    for (int c = 0; c < VC; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (16 * c + 4 * lg < dv) part[16 * c + 4 * lg + r] = acc[c][r];
    // the merge works with natural exponents
    if (lg == 0) { part[dv] = M == -INFINITY ? CA_NEG : M * 0.6931471805599453f; part[dv + 1] = L; }
    return;
  }
  const float inv = L > 0.f ? 1.0f / L : 0.f;
  float mul = inv;
  if constexpr (MAPS == 2) {
    if (wave == 1) hand(0, inv * a.lambda);
    __syncthreads();
    if (wave != 0) return;
#pragma unroll
    for (int c = 0; c < VC; ++c) acc[c] *= inv;
    take(0, -1.f);
    float q2 = 0.f;
#pragma unroll
    for (int c = 0; c < VC; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) q2 += 16 * c + 4 * lg < dv ? acc[c][r] * acc[c][r] : 0.f;
    q2 += __shfl_xor(q2, 16, 64);
    q2 += __shfl_xor(q2, 32, 64);
    mul = a.out_scale / sqrtf(q2 / (float)dv + a.eps);
  }
  if (wave != 0 || li >= nh) return;
  const T* gt = (const T*)a.gate + t * a.gate_token_stride;
  if (a.gate != nullptr && !a.gate_per_feature) mul *= ca_sigmoid_fast(to_f32(gt[h]));
  T* op = (T*)a.out + t * a.out_token_stride + (int64_t)h * dv;
#pragma unroll
  for (int c = 0; c < VC; ++c) {
    const int col = 16 * c + 4 * lg;
    if (col >= dv) continue;
    Vec<T, 4> w;
    if (a.gate != nullptr && a.gate_per_feature) {
      const Vec<T, 4> z = ldvec<T, 4>(gt + (int64_t)h * dv + col);
#pragma unroll
      for (int r = 0; r < 4; ++r) w.v[r] = from_f32<T>(acc[c][r] * mul * ca_sigmoid_fast(to_f32(z.v[r])));
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) w.v[r] = from_f32<T>(acc[c][r] * mul);
    }
    stvec<T, 4>(op + col, w);
  }
}

// ------------------------------------------------------------------------------------------------ launches
inline bool ca_matrix_shape(int dtype, int maps, int d, int dv) {
  return (dtype == MI355_BF16 || dtype == MI355_F16) && d % 8 == 0 && dv % 8 == 0 && d <= (maps == 2 ? 128 : 256) && dv <= 256;
}
inline int ca_rows(int dtype, int maps, int d, int dv) { return ca_matrix_shape(dtype, maps, d, dv) ? (maps == 2 ? 64 : 128) : CV_ROWS; }

template <typename T, int KS, int VT, int MAPS> int launch_ca_tile(const CaArgs& a, hipStream_t st) {
  constexpr size_t lds = ca_tile_lds<KS, VT, MAPS>();
  const int rep = a.heads / a.kv_heads, chunks = (rep + a.rows_heads - 1) / a.rows_heads;
  const int64_t wgs = a.num_runs * a.kv_heads * chunks;
  MI355_REQUIRE(wgs < ((int64_t)1 << 31), MI355_ERR_UNSUPPORTED, "causal_attention: too many runs");
  auto go = [&](auto kern) -> int {
    if (lds > 64 * 1024) {
      hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      MI355_REQUIRE(e == hipSuccess, MI355_ERR_LAUNCH, "causal_attention: %zu bytes of LDS refused", lds);
    }
    hipLaunchKernelGGL(kern, dim3((unsigned)wgs), dim3(256), lds, st, a);
    return MI355_OK;
  };
  return a.cap > 0.f ? go(causal_attention_tile_kernel<T, KS, VT, MAPS, true>) : go(causal_attention_tile_kernel<T, KS, VT, MAPS, false>);
}
template <typename T, int KS, int VC, int MAPS> int launch_ca_token(const CaArgs& a, hipStream_t st) {
  constexpr size_t lds = ct_lds<VC>();
  const int rep = a.heads / a.kv_heads;
  const int64_t wgs = a.num_runs * a.kv_heads * ((rep + 15) / 16);
  MI355_REQUIRE(wgs < ((int64_t)1 << 31), MI355_ERR_UNSUPPORTED, "causal_attention: too many tokens");
  auto kern = causal_attention_token_kernel<T, KS, VC, MAPS>;
  if (lds > 64 * 1024) {
    hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    MI355_REQUIRE(e == hipSuccess, MI355_ERR_LAUNCH, "causal_attention: %zu bytes of LDS refused", lds);
  }
  hipLaunchKernelGGL(kern, dim3((unsigned)wgs, (unsigned)a.num_splits), dim3(256), lds, st, a);
  return MI355_OK;
}

template <typename T, int MAPS> int launch_ca_matrix(const CaArgs& a, bool single, hipStream_t st) {
  const int d = a.d, dv = a.dv;
#define MI355_CA_V(FN, KS, A, B, C)                                     \
  (dv <= 64 ? FN<T, KS, A, MAPS>(a, st) : dv <= 128 ? FN<T, KS, B, MAPS>(a, st) : FN<T, KS, C, MAPS>(a, st))
  if (single) {
    if (d <= 64) return MI355_CA_V(launch_ca_token, 2, 4, 8, 16);
    if (d <= 128) return MI355_CA_V(launch_ca_token, 4, 4, 8, 16);
    if constexpr (MAPS == 1) return MI355_CA_V(launch_ca_token, 8, 4, 8, 16);
  } else {
    if (d <= 64) return MI355_CA_V(launch_ca_tile, 4, 2, 4, 8);
    if (d <= 128) return MI355_CA_V(launch_ca_tile, 8, 2, 4, 8);
    if constexpr (MAPS == 1) return MI355_CA_V(launch_ca_tile, 16, 2, 4, 8);
  }
#undef MI355_CA_V
  set_error("causal_attention: head width %d not served", d);
  return MI355_ERR_UNSUPPORTED;
}

template <typename T, int MAPS> int launch_ca_valu(const CaArgs& a, hipStream_t st) {
  const int rep = a.heads / a.kv_heads, chunks = (rep + a.rows_heads - 1) / a.rows_heads;
  const int w = MAPS * a.d;
  const size_t lds = ((size_t)CV_ROWS * w + (size_t)CV_KT * (w + 1) + (size_t)CV_KT * a.dv + (size_t)MAPS * CV_ROWS * CV_KT) * sizeof(float);
  MI355_REQUIRE(lds <= 160 * 1024, MI355_ERR_UNSUPPORTED, "causal_attention: head widths %d x %d / %d together need %zu bytes of LDS", MAPS, a.d,
                a.dv, lds);
  MI355_REQUIRE(a.kv_heads * chunks <= 65535 && a.num_runs < ((int64_t)1 << 31), MI355_ERR_UNSUPPORTED, "causal_attention: too many heads or runs");
  const dim3 grid((unsigned)a.num_runs, (unsigned)(a.kv_heads * chunks), (unsigned)a.num_splits);
  auto go = [&](auto kern) -> int {
    if (lds > 64 * 1024) {
      hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      MI355_REQUIRE(e == hipSuccess, MI355_ERR_LAUNCH, "causal_attention: %zu bytes of LDS refused", lds);
    }
    hipLaunchKernelGGL(kern, grid, dim3(256), lds, st, a);
    return MI355_OK;
  };
  return a.dv <= 128 ? go(causal_attention_valu_kernel<T, MAPS, 8>) : go(causal_attention_valu_kernel<T, MAPS, 32>);
}

template <typename T, int MAPS> int launch_ca(const CaArgs& a, bool matrix, bool single, hipStream_t st) {
  int rc;
  if constexpr (!std::is_same<T, float>::value) rc = matrix ? launch_ca_matrix<T, MAPS>(a, single, st) : launch_ca_valu<T, MAPS>(a, st);
  else rc = launch_ca_valu<T, MAPS>(a, st);
  if (rc != MI355_OK) return rc;
  MI355_CHECK_LAUNCH("causal_attention");
  if (a.num_splits > 1) {
    hipLaunchKernelGGL((causal_attention_merge_kernel<T, MAPS>), dim3((unsigned)((a.num_runs * a.heads + 3) / 4)), dim3(256), 0, st, a);
    MI355_CHECK_LAUNCH("causal_attention(merge)");
  }
  return MI355_OK;
}

}  // namespace
}  // namespace mi355

using namespace mi355;

int mi355_causal_attention_run_tokens(int heads, int kv_heads, int maps, int head_dim, int v_head_dim, int dtype) {
  if (heads <= 0 || kv_heads <= 0 || heads % kv_heads || maps < 1 || maps > 2) return 0;
  const int rows = ca_rows(dtype, maps, head_dim, v_head_dim);
  return std::max(1, rows / std::min(heads / kv_heads, rows));
}

int mi355_causal_attention(void* out, const void* q, const void* k_cache, const void* v_cache, const int32_t* req_to_token,
                           const int64_t* req_pool_indices, const int32_t* tok_req, const int64_t* positions, const int32_t* runs,
                           int64_t num_runs, const void* gate, int gate_per_feature, int64_t gate_token_stride, int64_t q_token_stride,
                           int64_t out_token_stride, int64_t req_to_token_stride, int heads, int kv_heads, int maps, int head_dim,
                           int v_head_dim, float scale, float cap, float lambda, float out_scale, float eps, int num_splits,
                           float* split_scratch, int64_t tokens, int max_run, int dtype, void* stream) {
  MI355_REQUIRE(out && q && k_cache && v_cache && req_to_token && req_pool_indices && positions, MI355_ERR_INVALID,
                "causal_attention: null pointer");
  MI355_REQUIRE(heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && head_dim > 0 && v_head_dim > 0 && tokens >= 0 && num_runs >= 0 &&
                    (maps == 1 || maps == 2) && scale > 0.f && cap >= 0.f, MI355_ERR_INVALID, "causal_attention: bad shape or scale");
  MI355_REQUIRE(q_token_stride >= (int64_t)heads * maps * head_dim && out_token_stride >= (int64_t)heads * v_head_dim, MI355_ERR_INVALID,
                "causal_attention: rows of q or of the result overlap");
  MI355_REQUIRE(gate == nullptr || gate_token_stride >= (gate_per_feature ? (int64_t)heads * v_head_dim : heads), MI355_ERR_INVALID,
                "causal_attention: bad gate stride");
  MI355_REQUIRE(runs != nullptr ? (tok_req != nullptr) : (num_runs == tokens), MI355_ERR_INVALID,
                "causal_attention: runs come with the tokens' sequences; without runs, one per token");
  MI355_REQUIRE(max_run >= 1 && num_splits >= 1 && num_splits <= 64 && (num_splits == 1 || (split_scratch && max_run == 1)), MI355_ERR_INVALID,
                "causal_attention: key ranges serve single tokens and need scratch");
  // per-map widths: K and Q tiles of the vector-ALU kernel must fit LDS
  MI355_REQUIRE((int64_t)maps * head_dim <= 512 && v_head_dim <= 512, MI355_ERR_UNSUPPORTED, "causal_attention: head width %d x %d / %d not served",
                maps, head_dim, v_head_dim);
  if (num_runs == 0) return MI355_OK;
  CaArgs a;
  a.out = out; a.q = q; a.k_cache = k_cache; a.v_cache = v_cache; a.req_to_token = req_to_token; a.req_pool_indices = req_pool_indices;
  a.tok_req = tok_req; a.positions = positions; a.runs = runs; a.gate = gate; a.partial = split_scratch; a.num_runs = num_runs;
  a.q_token_stride = q_token_stride; a.out_token_stride = out_token_stride; a.gate_token_stride = gate_token_stride;
  a.req_to_token_stride = req_to_token_stride; a.tokens = tokens; a.heads = heads; a.kv_heads = kv_heads; a.d = head_dim; a.dv = v_head_dim;
  a.gate_per_feature = gate_per_feature; a.num_splits = num_splits; a.scale = scale; a.cap = cap; a.lambda = lambda;
  a.out_scale = out_scale; a.eps = eps;
  // the matrix-core kernels need 16-byte rows of q, keys and values and 8-byte rows of the gate and the result; a caller whose
  // tensors are laid out otherwise gets the vector-ALU kernel, whose runs are shorter (max_run says how long the caller's are)
  const bool matrix = ca_matrix_shape(dtype, maps, head_dim, v_head_dim) && q_token_stride % 8 == 0 && aligned16(q) && aligned16(k_cache) &&
                      aligned16(v_cache) && aligned16(out) && out_token_stride % 4 == 0 &&
                      (gate == nullptr || !gate_per_feature || (gate_token_stride % 4 == 0 && reinterpret_cast<uintptr_t>(gate) % 8 == 0));
  const bool single = max_run == 1;
  const int rows = matrix ? (maps == 2 ? 64 : 128) : CV_ROWS;
  a.rows_heads = std::min(heads / kv_heads, rows);
  MI355_REQUIRE(max_run <= std::max(1, rows / a.rows_heads), MI355_ERR_UNSUPPORTED, "causal_attention: runs of up to %d tokens, this launch takes %d",
                max_run, std::max(1, rows / a.rows_heads));
  int rc = MI355_OK;
  MI355_DISPATCH_DTYPE(dtype, "causal_attention", {
    rc = maps == 2 ? launch_ca<T, 2>(a, matrix, single, (hipStream_t)stream) : launch_ca<T, 1>(a, matrix, single, (hipStream_t)stream);
  });
  return rc;
}
