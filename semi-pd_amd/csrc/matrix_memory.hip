// Matrix memory with exponential gates (mLSTM) over a pool of per-request state rows (gfx950, wave64).
//
// Rows of the projection hold q [H D], k [H D], v [H E], an output gate g [H E], and one input and one forget gate per head.
// Per head, with S [D, E] and n [D] from zero and a running maximum m from 0, all fp32:
//     i_t = cap tanh((i + b_i) / cap);   f_t = log sigmoid(cap tanh((f + b_f) / cap));   m_t = max(f_t + m_(t-1), i_t)
//     S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T;   n_t likewise with k_t alone
//     o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6),  q scaled by D^(-1/2)
// then every head's o to unit RMS (eps inside the root), times a weight over all heads, times sigmoid(g).
//
// The state row of a request: S of all heads [H, D, E] | n [H, D] | m [H].  A sequence's first rows start from zero whatever
// the row holds; otherwise the state is read before a launch's rows and written back behind them, so prompts cut into portions,
// single decode tokens and rows that change hands take one path.
//
//  * memory_chunk_kernel (bf16): prompt batches, 64 tokens at a time on the matrix cores.  With b_t the running sum of f inside
//    the chunk, a_s = i_s - b_s, m_t = b_t + max(m_in, max_(s <= t) a_s):
//        S_t^T q_t = exp(b_t + m_in - m_t) S_in^T q_t + sum_(s <= t) exp(a_s + b_t - m_t) (q_t . k_s) v_s
//    -- the same m_t, S and n as token by token, no exponent above 0.  q, k and v ARE bf16; the fp32 factors -- S, the weighted
//    scores, the weighted values -- enter the products as two bf16 terms each (high part and remainder, 16 bits of mantissa),
//    sums are fp32, and S itself stays in fp32 accumulators for the whole walk.  One workgroup per (request, head, 32 columns
//    of S); the next chunk's rows are in flight in registers during a chunk's products.  What depends on the gates alone --
//    b, a, the running maximum of a inside the chunk -- comes from memory_gate_kernel, once for all columns of a head.
//  * memory_scan_kernel: every element type and size, token by token, one wave per (request, head, 64 / NS columns of [S | n]).
//  * memory_step_kernel: batches of one token per request, a workgroup per (request, head, 64 columns): S is read and written
//    once, 16-byte accesses, every load of a thread in flight before the first is used.
//  * memory_out_kernel: the division, the norm of every head, the weight and the gate, a wave per (token, head).
#include "common.h"
#include "mfma_frag.h"

namespace semipd {

struct MemArgs {
  const void* p; int64_t ld;                              // projection rows
  int64_t q_off, k_off, v_off, g_off, i_off, f_off;       // their columns
  const float* i_bias; const float* f_bias;               // [H]
  float cap;
  float* work; int64_t wld;                               // fp32 [T, wld]: S^T q [H E] | n . q [H] | m [H]
  float* planes;                                          // fp32 [kMemPlanes, H, T] (memory_gate_kernel)
  float* state; int64_t state_ld;                         // fp32 [slots, >= H D E + H D + H]
  const int64_t* state_indices; const int64_t* seq_lens;
  const int32_t* q_start; const int32_t* q_len;           // [B] or NULL (one row per request)
  int64_t batch, num_tokens;
  int H, D, E;
  float q_scale;
  const void* norm_w; float eps;                          // [H E] of the activation type
  void* out; int64_t out_ld;                              // [T, H E] of the activation type
};

__device__ __forceinline__ float soft_cap(float x, float cap) { return cap * tanhf(x / cap); }
__device__ __forceinline__ float log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }

template <typename T>
__device__ __forceinline__ void memory_gates(const MemArgs& a, int64_t t, int h, float& i, float& f) {
  const T* p = (const T*)a.p + t * a.ld;
  i = soft_cap(Elem<T>::to_f(p[a.i_off + h]) + a.i_bias[h], a.cap);
  f = log_sigmoid(soft_cap(Elem<T>::to_f(p[a.f_off + h]) + a.f_bias[h], a.cap));
}

// the rows of request b in this launch: first row, how many, position of the first
__device__ __forceinline__ bool memory_rows(const MemArgs& a, int b, int64_t& t0, int64_t& n, int64_t& first_pos) {
  if (a.q_start == nullptr) {
    t0 = b; n = 1; first_pos = a.seq_lens[b] - 1;
  } else {
    t0 = a.q_start[b]; n = a.q_len[b]; first_pos = a.seq_lens[b] - n;
  }
  return n > 0 && first_pos >= 0;
}

// ---------------------------------------------------------------------------------- prompt batches on the matrix cores
constexpr int kMemChunk = 64;       // tokens of a chunk
constexpr int kMemCols = 32;        // columns of S of a workgroup
constexpr float kMemLog2e = 1.4426950408889634f;


// Inclusive scan over the 64 lanes in register moves (row shifts inside 16 lanes, then the last lane of a row to the rows behind)
template <int CTRL, int ROWS> __device__ __forceinline__ float dpp_or(float identity, float x) {
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, identity), __builtin_bit_cast(int, x), CTRL, ROWS,
                                                               0xf, false));
}
template <typename Op> __device__ __forceinline__ float row_scan(float x, float identity, Op op) {      // inside 16 lanes
  x = op(x, dpp_or<0x111, 0xf>(identity, x));
  x = op(x, dpp_or<0x112, 0xf>(identity, x));
  x = op(x, dpp_or<0x114, 0xf>(identity, x));
  return op(x, dpp_or<0x118, 0xf>(identity, x));
}
template <typename Op> __device__ __forceinline__ float rows_scan(float x, float identity, Op op) {     // over the rows behind it
  x = op(x, dpp_or<0x142, 0xa>(identity, x));      // lane 15 -> row 1, lane 47 -> row 3
  return op(x, dpp_or<0x143, 0xc>(identity, x));   // lane 31 -> rows 2 and 3
}
__device__ __forceinline__ float lane_value(float x, int lane) {
  return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, x), lane));
}

// What the gates of a chunk come to, a wave per (chunk, head), lane = token; logarithms to base 2.  Planes: 0 b (running sum of
// the log forget gates), 1 a = i - b, 2 the running maximum of a, 3 the maximum A of a over the token's tile of 16, 4
// exp2(a - A).  Tokens past the end are not written.
constexpr int kMemPlanes = 5;
__global__ void __launch_bounds__(256) memory_gate_kernel(MemArgs a) {
  const int lane = threadIdx.x & 63, h = blockIdx.y * 4 + (threadIdx.x >> 6);
  if (h >= a.H) return;
  int64_t left = blockIdx.x;
  int b = 0;
  for (; b < (int)a.batch; ++b) {
    const int64_t chunks = ((int64_t)a.q_len[b] + kMemChunk - 1) / kMemChunk;
    if (left < chunks) break;
    left -= chunks;
  }
  if (b >= (int)a.batch) return;
  const int64_t at_row = left * kMemChunk + lane, t = a.q_start[b] + at_row;
  const bool there = at_row < a.q_len[b];
  float i = -INFINITY, f = 0.f;
  if (there) memory_gates<bf16_t>(a, t, h, i, f);
  auto add = [](float x, float y) { return x + y; };
  auto max2 = [](float x, float y) { return fmaxf(x, y); };
  const float bs = rows_scan(row_scan(f * kMemLog2e, 0.f, add), 0.f, add);
  const float as = i * kMemLog2e - bs;
  const float in_tile = row_scan(as, -INFINITY, max2);
  const float run = rows_scan(in_tile, -INFINITY, max2);
  const float top = __shfl(in_tile, lane | 15, 64);
  if (!there) return;
  const int64_t step = (int64_t)a.H * a.num_tokens;
  float* w = a.planes + (int64_t)h * a.num_tokens + t;
  w[0] = bs;
  w[step] = as;
  w[2 * step] = run;
  w[3 * step] = top;
  w[4 * step] = __builtin_amdgcn_exp2f(as - top);
}

// x as its upper 16 bits and the bf16 of what they leave of it (the upper bits of two numbers are one byte permutation)
__device__ __forceinline__ void split_pair(float x0, float x1, uint32_t& hi, uint32_t& lo) {
  const uint32_t w0 = __float_as_uint(x0), w1 = __float_as_uint(x1);
  hi = __builtin_amdgcn_perm(w1, w0, 0x07060302u);
  lo = pack2<bf16_t>(x0 - __uint_as_float(w0 & 0xffff0000u), x1 - __uint_as_float(w1 & 0xffff0000u));
}

__host__ __device__ constexpr int mem_k_stride(int nd) { return nd * 64 + 32; }       // bytes of a row of the K tile and of S^T
constexpr int kMemVStride = 96;                                                        // of the V tile

template <int ND> constexpr size_t mem_chunk_lds() {
  return (size_t)kMemChunk * mem_k_stride(ND) + 2 * (size_t)kMemCols * mem_k_stride(ND) + kMemChunk * kMemVStride +
         32 * ND * (sizeof(float) + 2 * sizeof(uint16_t)) + 3 * kMemChunk * sizeof(float);
}

// What a wave's 16 queries see: o += S^T q (two 16-row tiles, high and low parts), dn += n q (WITH_N; row 0 of the result) and
// sc[t] = k q of the first NT key tiles, in walks over the key elements in which the operands of the next 32 elements are on
// their way out of LDS while the current ones are multiplied.  (Two walks hold half the operands each.)
template <int ND, int NT, bool WITH_S, bool WITH_N>
__device__ __forceinline__ void read_products(const uint8_t* k_row, const uint8_t* sh_row, const uint8_t* sl_row, const uint8_t* n_row,
                                              const Frag16 (&qf)[ND], f32x4 (&o)[2], f32x4 (&sc)[4], f32x4& dn) {
  constexpr int RSK = mem_k_stride(ND), S0 = WITH_S ? 4 : 0, N0 = S0 + NT, F = N0 + (WITH_N ? 2 : 0);
  Frag16 fa[F], fb[F];
  auto load = [&](int kk, Frag16 (&x)[F]) {
    if constexpr (WITH_S) {
      x[0].u = *reinterpret_cast<const uint4*>(sh_row + kk * 64);
      x[1].u = *reinterpret_cast<const uint4*>(sh_row + 16 * RSK + kk * 64);
      x[2].u = *reinterpret_cast<const uint4*>(sl_row + kk * 64);
      x[3].u = *reinterpret_cast<const uint4*>(sl_row + 16 * RSK + kk * 64);
    }
#pragma unroll
    for (int t = 0; t < NT; ++t) x[S0 + t].u = *reinterpret_cast<const uint4*>(k_row + 16 * t * RSK + kk * 64);
    if constexpr (WITH_N) {
      x[N0].u = *reinterpret_cast<const uint4*>(n_row + kk * 64);
      x[N0 + 1].u = *reinterpret_cast<const uint4*>(n_row + 64 * ND + kk * 64);
    }
  };
  auto mul = [&](const Frag16& q, const Frag16 (&x)[F]) {
    if constexpr (WITH_S) {
      o[0] = mma16<bf16_t>(x[0], q, o[0]);
      o[1] = mma16<bf16_t>(x[1], q, o[1]);
    }
    if constexpr (WITH_N) dn = mma16<bf16_t>(x[N0], q, dn);
#pragma unroll
    for (int t = 0; t < NT; ++t) sc[t] = mma16<bf16_t>(x[S0 + t], q, sc[t]);
    if constexpr (WITH_S) {
      o[0] = mma16<bf16_t>(x[2], q, o[0]);
      o[1] = mma16<bf16_t>(x[3], q, o[1]);
    }
    if constexpr (WITH_N) dn = mma16<bf16_t>(x[N0 + 1], q, dn);
  };
  load(0, fa);
#pragma unroll
  for (int kk = 0; kk < ND; kk += 2) {
    load(kk + 1, fb);
    __builtin_amdgcn_sched_barrier(0);
    mul(qf[kk], fa);
    __builtin_amdgcn_sched_barrier(0);
    if (kk + 2 < ND) load(kk + 2, fa);
    __builtin_amdgcn_sched_barrier(0);
    mul(qf[kk + 1], fb);
    __builtin_amdgcn_sched_barrier(0);
  }
}

template <int ND>          // key sizes up to 32 * ND, ND even
__global__ void __launch_bounds__(256, 2) memory_chunk_kernel(MemArgs a) {
  extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
  constexpr int RSK = mem_k_stride(ND), DT = ND / 2, NK = ND;      // DT: 16-row tiles of S per wave; NK: 16-byte K pieces per thread
  uint8_t* k_lds = lds;
  uint8_t* s_hi = k_lds + kMemChunk * RSK;
  uint8_t* s_lo = s_hi + kMemCols * RSK;
  uint8_t* v_lds = s_lo + kMemCols * RSK;
  float* n_lds = reinterpret_cast<float*>(v_lds + kMemChunk * kMemVStride);      // n as the chunk finds it [32 ND]
  uint8_t* nb_lds = reinterpret_cast<uint8_t*>(n_lds + 32 * ND);                 // the same as high and low bf16 parts [2][32 ND]
  float* a_lds = reinterpret_cast<float*>(nb_lds + 128 * ND);                    // a_s [64]
  float* x_lds = a_lds + kMemChunk;                                              // exp2(a_s - maximum of the tile) [64]
  float* u_lds = x_lds + kMemChunk;                                              // exp2(a_s + b_last - m_out) [64]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 15, g = lane >> 4;
  const int H = a.H, D = a.D, E = a.E;
  const int slices = (E + kMemCols - 1) / kMemCols;
  // consecutive workgroup ids go round the eight XCDs: an XCD takes a contiguous range of items, so the slices of a head --
  // which read the same q and k -- share an L2 (gridDim.x is a multiple of 8)
  const int64_t n_items = gridDim.x, item = (int64_t)(blockIdx.x & 7) * (n_items >> 3) + (blockIdx.x >> 3);
  if (item >= a.batch * H * slices) return;
  const int sl = (int)(item % slices), h = (int)(item / slices % H), b = (int)(item / slices / H);
  int64_t t0, n, first_pos;
  if (!memory_rows(a, b, t0, n, first_pos)) return;
  const bool fresh = first_pos == 0, lead = sl == 0;       // the first slice keeps n and m and writes n . q
  const int e0 = sl * kMemCols;
  const bf16_t* p = (const bf16_t*)a.p + t0 * a.ld;
  float* work = a.work + t0 * a.wld;
  float* st = a.state + a.state_indices[b] * a.state_ld;
  float* stS = st + (int64_t)h * D * E;
  float* stn = st + (int64_t)H * D * E + (int64_t)h * D;
  float* stm = st + (int64_t)H * D * E + (int64_t)H * D + h;

  // S of this workgroup in accumulators: rows d = 16 (DT wave + dt) + 4 g + i, column e0 + 16 et + r; n in LDS
  f32x4 acc[DT][2];
  float m_in = fresh ? 0.f : *stm * kMemLog2e;              // logarithms to base 2, as in the planes
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * (DT * wave + dt) + 4 * g + i;
#pragma unroll
      for (int et = 0; et < 2; ++et) {
        const int e = e0 + 16 * et + r;
        acc[dt][et][i] = (!fresh && d < D && e < E) ? stS[(int64_t)d * E + e] : 0.f;
      }
    }
  if (lead && tid < 32 * ND) n_lds[tid] = (!fresh && tid < D) ? stn[tid] : 0.f;

  // The rows of a chunk.  Rows past the end are the last row once more and elements past D (E) the first ones: finite numbers whose
  // weights are zero (queries are zero past D; results past E and rows past the end are not stored).  Every address is a
  // pointer of the workgroup plus 32 bits of the thread.
  constexpr int KR = 64 / ND;                        // piece i of the K tile that this thread moves: row k_row + KR i
  const int k_row = tid / (4 * ND), k_d = (tid % (4 * ND)) * 8;
  const int v_e = (tid & 3) * 8;
  const uint8_t* kp = reinterpret_cast<const uint8_t*>(p + a.k_off + (int64_t)h * D);
  const uint8_t* vp = reinterpret_cast<const uint8_t*>(p + a.v_off + (int64_t)h * E + e0);
  const uint8_t* qp = reinterpret_cast<const uint8_t*>(p + a.q_off + (int64_t)h * D);
  const float* gp = a.planes + (int64_t)h * a.num_tokens + t0;
  const int64_t g_step = (int64_t)H * a.num_tokens;
  const uint32_t ldb = (uint32_t)a.ld * 2;           // bytes of a row
  const uint32_t k_col = (uint32_t)(k_d < D ? k_d : 0) * 2, v_col = (uint32_t)(e0 + v_e < E ? v_e : 0) * 2;
  const uint32_t k_voff = k_row * ldb + k_col, v_voff = (tid >> 2) * ldb + v_col, q_row = (16 * wave + r) * ldb;
  u32x4 kr[NK], vr;
  Frag16 qf[ND];
  float gl[kMemPlanes];           // the planes' values of token `lane`
  auto fetch = [&](int64_t c0) {
    const int last = (int)(n - c0 < kMemChunk ? n - c0 : kMemChunk) - 1;
    const uint8_t* kc = kp + c0 * ldb;
    const uint8_t* vc = vp + c0 * ldb;
    if (last == kMemChunk - 1) {
#pragma unroll
      for (int i = 0; i < NK; ++i) kr[i] = *reinterpret_cast<const u32x4*>(kc + (int64_t)(i * KR) * ldb + k_voff);
      vr = *reinterpret_cast<const u32x4*>(vc + v_voff);
    } else {
#pragma unroll
      for (int i = 0; i < NK; ++i) {
        const int row = k_row + i * KR;
        kr[i] = *reinterpret_cast<const u32x4*>(kc + ((row < last ? row : last) * ldb + k_col));
      }
      const int row = tid >> 2;
      vr = *reinterpret_cast<const u32x4*>(vc + ((row < last ? row : last) * ldb + v_col));
    }
    const uint32_t gr = lane < last ? lane : last;
#pragma unroll
    for (int x = 0; x < kMemPlanes; ++x) gl[x] = gp[x * g_step + c0 + gr];
  };
  auto fetch_q = [&](int64_t c0) {      // straight into the operand registers, once the chunk in front has used them
    const int last = (int)(n - c0 < kMemChunk ? n - c0 : kMemChunk) - 1;
    const uint8_t* qc = qp + c0 * ldb;
    const uint32_t voff = 16 * wave + r <= last ? q_row : last * ldb;
#pragma unroll
    for (int kk = 0; kk < ND; ++kk) {
      const int d = 32 * kk + 8 * g;
      qf[kk].u = *reinterpret_cast<const uint4*>(qc + (voff + (d < D ? d : 0) * 2));
    }
  };
  fetch(0);
  fetch_q(0);
  for (int64_t c0 = 0; c0 < n; c0 += kMemChunk) {
    const int cnt = (int)(n - c0 < kMemChunk ? n - c0 : kMemChunk);
    // the chunk's gates, in every wave: lane = token (lanes past the end hold the last token's)
    const float bt = gl[0], at = gl[1], mt = bt + fmaxf(m_in, gl[2]);
    const float b_last = lane_value(bt, 63), m_out = lane_value(mt, 63);
    const float keep = __builtin_amdgcn_exp2f(b_last + m_in - m_out);
    float tile_top[3];                   // maximum of a over the tiles of 16 tokens that later tiles look back at
#pragma unroll
    for (int t = 0; t < 3; ++t) tile_top[t] = lane_value(gl[3], 16 * t);

    __syncthreads();                     // everyone is done with the tiles of the chunk in front
#pragma unroll
    for (int i = 0; i < NK; ++i) *reinterpret_cast<u32x4*>(k_lds + (k_row + KR * i) * RSK + k_d * 2) = kr[i];
    *reinterpret_cast<u32x4*>(v_lds + (tid >> 2) * kMemVStride + (tid & 3) * 16) = vr;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const int d0 = 16 * (DT * wave + dt) + 4 * g;
#pragma unroll
      for (int et = 0; et < 2; ++et) {
        uint2 hi, lo;
        split_pair(acc[dt][et][0], acc[dt][et][1], hi.x, lo.x);
        split_pair(acc[dt][et][2], acc[dt][et][3], hi.y, lo.y);
        *reinterpret_cast<uint2*>(s_hi + (16 * et + r) * RSK + d0 * 2) = hi;
        *reinterpret_cast<uint2*>(s_lo + (16 * et + r) * RSK + d0 * 2) = lo;
      }
    }
    if (wave == 0) {
      a_lds[lane] = at;
      x_lds[lane] = gl[4];
      u_lds[lane] = lane < cnt ? __builtin_amdgcn_exp2f(at + b_last - m_out) : 0.f;
    }
    if (lead) {
      // (n_lds of this wave's own rows: written by its own lanes at the end of the chunk in front)
      const int pair = 8 * ND / 2 * wave + lane;
      if (lane < 4 * ND) {
        const float2 x = *reinterpret_cast<const float2*>(n_lds + 2 * pair);
        uint32_t hi, lo;
        split_pair(x.x, x.y, hi, lo);
        *reinterpret_cast<uint32_t*>(nb_lds + 4 * pair) = hi;
        *reinterpret_cast<uint32_t*>(nb_lds + 64 * ND + 4 * pair) = lo;
      }
    }
    if (32 * ND > D) {
#pragma unroll
      for (int kk = 0; kk < ND; ++kk)
        if (32 * kk + 8 * g >= D) qf[kk].u = uint4{0u, 0u, 0u, 0u};
    }
    __syncthreads();
    if (c0 + kMemChunk < n) fetch(c0 + kMemChunk);          // in flight during the products

    // this lane's query: row 16 wave + r of the chunk
    const int qr = 16 * wave + r;
    const float q_m = __shfl(mt, qr, 64), q_bm = __shfl(bt, qr, 64) - q_m;
    const float q_in = __builtin_amdgcn_exp2f(q_bm + m_in);
    f32x4 o[2], sc[4], dn = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < 4; ++t) sc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    o[0] = o[1] = dn;
    {
      const uint8_t* k_r = k_lds + r * RSK + g * 16;
      const uint8_t* sh_r = s_hi + r * RSK + g * 16;
      const uint8_t* sl_r = s_lo + r * RSK + g * 16;
      const uint8_t* n_r = nb_lds + g * 16;               // (the same row for every r: row 0 of the result is the one that counts)
      if (lead) read_products<ND, 0, true, true>(k_r, sh_r, sl_r, n_r, qf, o, sc, dn);
      else read_products<ND, 0, true, false>(k_r, sh_r, sl_r, n_r, qf, o, sc, dn);
      if (wave < 2) read_products<ND, 2, false, false>(k_r, sh_r, sl_r, n_r, qf, o, sc, dn);
      else read_products<ND, 4, false, false>(k_r, sh_r, sl_r, n_r, qf, o, sc, dn);
    }
    if (c0 + kMemChunk < n) fetch_q(c0 + kMemChunk);
    // values of the chunk, [e = 16 et + r][tokens 32 s + 4 g .. + 3 and 32 s + 16 + 4 g .. + 3]
    Frag16 va[2][2];
#pragma unroll
    for (int s = 0; s < 2; ++s)
#pragma unroll
      for (int et = 0; et < 2; ++et) {
        const uint8_t* vrow = v_lds + (32 * s + 4 * g + (r >> 2)) * kMemVStride + (r & 3) * 8 + et * 32;
        va[s][et].s[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)vrow);
        va[s][et].s[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(vrow + 16 * kMemVStride));
      }
    float den = dn[0] * q_in;                              // (lanes g == 0 hold row 0)
    den = g == 0 ? den : 0.f;
#pragma unroll
    for (int et = 0; et < 2; ++et)
#pragma unroll
      for (int i = 0; i < 4; ++i) o[et][i] *= q_in;
    // the tokens of the chunk up to the query: weighted scores straight into the product with the values
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      if (32 * s > 16 * wave + 15) break;
      Frag16 ph, pl;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const int kt = 2 * s + half;
        float w[4] = {0.f, 0.f, 0.f, 0.f};
        if (kt < wave) {
          // a tile in front of the query's: exp2(a_s - A) exp2(A + b_t - m_t), both at most 1
          const float4 xs = *reinterpret_cast<const float4*>(x_lds + 16 * kt + 4 * g);
          const float y = __builtin_amdgcn_exp2f(tile_top[kt < 3 ? kt : 0] + q_bm);
          w[0] = sc[kt][0] * xs.x * y;
          w[1] = sc[kt][1] * xs.y * y;
          w[2] = sc[kt][2] * xs.z * y;
          w[3] = sc[kt][3] * xs.w * y;
        } else if (kt == wave) {
          const float4 as = *reinterpret_cast<const float4*>(a_lds + 16 * kt + 4 * g);
          const float av[4] = {as.x, as.y, as.z, as.w};
#pragma unroll
          for (int i = 0; i < 4; ++i) w[i] = 4 * g + i <= r ? sc[kt][i] * __builtin_amdgcn_exp2f(av[i] + q_bm) : 0.f;
        }
        den += (w[0] + w[1]) + (w[2] + w[3]);
        split_pair(w[0], w[1], ph.w[2 * half], pl.w[2 * half]);
        split_pair(w[2], w[3], ph.w[2 * half + 1], pl.w[2 * half + 1]);
      }
#pragma unroll
      for (int et = 0; et < 2; ++et) o[et] = mma16<bf16_t>(va[s][et], ph, o[et]);
#pragma unroll
      for (int et = 0; et < 2; ++et) o[et] = mma16<bf16_t>(va[s][et], pl, o[et]);
    }
    if (qr < cnt) {
      float* w = work + (c0 + qr) * a.wld;
#pragma unroll
      for (int et = 0; et < 2; ++et) {
        const int e = e0 + 16 * et + 4 * g;
        if (e < E)
          *reinterpret_cast<float4*>(w + (int64_t)h * E + e) =
              float4{o[et][0] * a.q_scale, o[et][1] * a.q_scale, o[et][2] * a.q_scale, o[et][3] * a.q_scale};
      }
    }
    if (lead) {
      den += __shfl_xor(den, 16, 64);
      den += __shfl_xor(den, 32, 64);
      if (g == 0 && qr < cnt) {
        float* w = work + (c0 + qr) * a.wld + (int64_t)H * E;
        w[h] = den * a.q_scale;
        w[H + h] = q_m * 0.6931471805599453f;
      }
    }
    // S <- keep S + sum_s k_s (u_s v_s)^T
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        acc[dt][0][i] *= keep;
        acc[dt][1][i] *= keep;
      }
    f32x4 nd[DT];
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) nd[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      if (32 * s >= cnt) break;
      Frag16 kt[DT];
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const uint8_t* krow = k_lds + (32 * s + 4 * g + (r >> 2)) * RSK + (r & 3) * 8 + (DT * wave + dt) * 32;
        kt[dt].s[0] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)krow);
        kt[dt].s[1] = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(krow + 16 * RSK));
      }
      const float4 ua = *reinterpret_cast<const float4*>(u_lds + 32 * s + 4 * g);
      const float4 ub = *reinterpret_cast<const float4*>(u_lds + 32 * s + 16 + 4 * g);
      const float us[8] = {ua.x, ua.y, ua.z, ua.w, ub.x, ub.y, ub.z, ub.w};
      Frag16 vh[2], vl[2], uh, ul;
#pragma unroll
      for (int u = 0; u < 4; ++u) split_pair(us[2 * u], us[2 * u + 1], uh.w[u], ul.w[u]);
#pragma unroll
      for (int et = 0; et < 2; ++et)
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const uint32_t w = va[s][et].w[u];
          split_pair(__uint_as_float(w << 16) * us[2 * u], __uint_as_float(w & 0xffff0000u) * us[2 * u + 1], vh[et].w[u], vl[et].w[u]);
        }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int et = 0; et < 2; ++et) acc[dt][et] = mma16<bf16_t>(kt[dt], vh[et], acc[dt][et]);
#pragma unroll
      for (int dt = 0; dt < DT; ++dt)
#pragma unroll
        for (int et = 0; et < 2; ++et) acc[dt][et] = mma16<bf16_t>(kt[dt], vl[et], acc[dt][et]);
      if (lead) {           // n <- keep n + sum_s u_s k_s: the same product with u_s as every column
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) nd[dt] = mma16<bf16_t>(kt[dt], uh, nd[dt]);
#pragma unroll
        for (int dt = 0; dt < DT; ++dt) nd[dt] = mma16<bf16_t>(kt[dt], ul, nd[dt]);
      }
    }
    if (lead && r == 0) {   // column 0 is added to n of the wave's own rows
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        float4* np = reinterpret_cast<float4*>(n_lds + 16 * (DT * wave + dt) + 4 * g);
        const float4 x = *np;
        *np = float4{x.x * keep + nd[dt][0], x.y * keep + nd[dt][1], x.z * keep + nd[dt][2], x.w * keep + nd[dt][3]};
      }
    }
    m_in = m_out;
  }
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 16 * (DT * wave + dt) + 4 * g + i;
      if (d >= D) continue;
#pragma unroll
      for (int et = 0; et < 2; ++et) {
        const int e = e0 + 16 * et + r;
        if (e < E) stS[(int64_t)d * E + e] = acc[dt][et][i];
      }
    }
  if (lead) {
    __syncthreads();
    for (int d = tid; d < D; d += 256) stn[d] = n_lds[d];
  }
  // (every slice of this head has read m before its first chunk's barrier -- but in workgroups of their own: m goes to the work
  //  row of the portion's last token, and memory_keep_max_kernel takes it from there once all slices are done)
}

// the running maximum of every (request, head) behind the launch's last row, out of the work rows
__global__ void __launch_bounds__(64) memory_keep_max_kernel(MemArgs a) {
  const int64_t id = (int64_t)blockIdx.x * 64 + threadIdx.x;
  if (id >= a.batch * a.H) return;
  const int b = (int)(id / a.H), h = (int)(id % a.H);
  int64_t t0, n, first_pos;
  if (!memory_rows(a, b, t0, n, first_pos)) return;
  a.state[a.state_indices[b] * a.state_ld + (int64_t)a.H * a.D * a.E + (int64_t)a.H * a.D + h] =
      a.work[(t0 + n - 1) * a.wld + (int64_t)a.H * a.E + a.H + h];
}

// ---------------------------------------------------------------------------------- token by token, any type and size
// A column of [S | n] (column E is n, its "value" is 1) lives in the registers of NS adjacent lanes, NPT rows each.
template <typename T, int NPT, int NS>
__global__ void __launch_bounds__(64) memory_scan_kernel(MemArgs a, int stage) {
  extern __shared__ __attribute__((aligned(16))) float scan_l[];      // per staged token: q [NP] | k [NP] | v of the block's columns
  constexpr int NP = NPT * NS, COLS = 64 / NS, TOK = 2 * NP + COLS;
  const int lane = threadIdx.x, H = a.H, D = a.D, E = a.E;
  const int eblocks = (E + 1 + COLS - 1) / COLS;
  int64_t id = blockIdx.x;
  const int eb = (int)(id % eblocks); id /= eblocks;
  const int h = (int)(id % H), b = (int)(id / H);
  int64_t t0, n, first_pos;
  if (!memory_rows(a, b, t0, n, first_pos)) return;
  const bool fresh = first_pos == 0;
  const int col = lane / NS, ns = lane % NS, e = eb * COLS + col, d0 = ns * NPT;
  const bool e_ok = e <= E, is_n = e == E;
  float* st = a.state + a.state_indices[b] * a.state_ld;
  float* base = is_n ? st + (int64_t)H * D * E + (int64_t)h * D : st + (int64_t)h * D * E + e;
  const int64_t step = is_n ? 1 : E;
  const float* stm = st + (int64_t)H * D * E + (int64_t)H * D + h;
  float S[NPT];
#pragma unroll
  for (int i = 0; i < NPT; ++i) S[i] = (!fresh && e_ok && d0 + i < D) ? base[(d0 + i) * step] : 0.f;
  float m = fresh ? 0.f : *stm;
  const T* p = (const T*)a.p;
  for (int64_t s0 = 0; s0 < n; s0 += stage) {
    const int cnt = (int)(n - s0 < stage ? n - s0 : stage);
    float gi = 0.f, gf = 0.f;
    if (lane < cnt) memory_gates<T>(a, t0 + s0 + lane, h, gi, gf);
    __syncthreads();
    for (int it = lane; it < cnt * TOK; it += 64) {
      const int k = it / TOK, x = it % TOK;
      const T* row = p + (t0 + s0 + k) * a.ld;
      float v = 0.f;
      if (x < NP) {
        if (x < D) v = Elem<T>::to_f(row[a.q_off + (int64_t)h * D + x]);
      } else if (x < 2 * NP) {
        if (x - NP < D) v = Elem<T>::to_f(row[a.k_off + (int64_t)h * D + x - NP]);
      } else {
        const int ee = eb * COLS + x - 2 * NP;
        v = ee < E ? Elem<T>::to_f(row[a.v_off + (int64_t)h * E + ee]) : (ee == E ? 1.0f : 0.f);
      }
      scan_l[it] = v;
    }
    __syncthreads();
    for (int k = 0; k < cnt; ++k) {
      const float it = __shfl(gi, k, 64), ft = __shfl(gf, k, 64);
      const float m_new = fmaxf(ft + m, it);
      const float keep = expf(ft + m - m_new), add = expf(it - m_new);
      m = m_new;
      const float* l = scan_l + k * TOK;
      const float av = add * l[2 * NP + col];
      float y = 0.f;
#pragma unroll
      for (int i = 0; i < NPT; ++i) {
        S[i] = keep * S[i] + l[NP + d0 + i] * av;
        y += S[i] * l[d0 + i];
      }
#pragma unroll
      for (int o = 1; o < NS; o <<= 1) y += __shfl_xor(y, o, 64);
      if (ns == 0 && e_ok) {
        float* w = a.work + (t0 + s0 + k) * a.wld;
        if (is_n) {
          w[(int64_t)H * E + h] = y * a.q_scale;
          w[(int64_t)H * E + H + h] = m;
        } else {
          w[(int64_t)h * E + e] = y * a.q_scale;
        }
      }
    }
  }
  if (e_ok) {
#pragma unroll
    for (int i = 0; i < NPT; ++i)
      if (d0 + i < D) base[(d0 + i) * step] = S[i];
  }
}

// ---------------------------------------------------------------------------------- one token per request
// Thread (column group, row group): VEC adjacent columns, every 16th row of S.  The first slice of a head also keeps n.
template <typename T, int VEC>
__global__ void __launch_bounds__(256) memory_step_kernel(MemArgs a) {
  extern __shared__ __attribute__((aligned(16))) float step_l[];     // q [D] | k [D] | partial sums [16][16 VEC]
  __shared__ float red[16];
  constexpr int COLS = 16 * VEC, BATCH = 16;
  const int tid = threadIdx.x, H = a.H, D = a.D, E = a.E;
  const int b = blockIdx.z, h = blockIdx.y, e0 = blockIdx.x * COLS;
  const int64_t first_pos = a.seq_lens[b] - 1;
  if (first_pos < 0) return;
  const bool fresh = first_pos == 0, lead = blockIdx.x == 0;
  const T* row = (const T*)a.p + (int64_t)b * a.ld;
  float* st = a.state + a.state_indices[b] * a.state_ld;
  float* stS = st + (int64_t)h * D * E;
  float* stn = st + (int64_t)H * D * E + (int64_t)h * D;
  float* stm = st + (int64_t)H * D * E + (int64_t)H * D + h;
  float* ql = step_l;
  float* kl = step_l + D;
  float* part = step_l + (2 * D + 3) / 4 * 4;
  const int cg = tid & 15, rg = tid >> 4, e = e0 + cg * VEC;
  const bool e_ok = e < E;
  // the first BATCH rows' state is asked for before anything waits
  float S[BATCH][VEC];
  auto load = [&](int i0) {
#pragma unroll
    for (int i = 0; i < BATCH; ++i) {
      const int d = rg + 16 * (i0 + i);
      if (!fresh && e_ok && d < D) {
        if constexpr (VEC == 4) {
          const float4 x = *reinterpret_cast<const float4*>(stS + (int64_t)d * E + e);
          S[i][0] = x.x; S[i][1] = x.y; S[i][2] = x.z; S[i][3] = x.w;
        } else {
          S[i][0] = stS[(int64_t)d * E + e];
        }
      } else {
#pragma unroll
        for (int u = 0; u < VEC; ++u) S[i][u] = 0.f;
      }
    }
  };
  load(0);
  float it, ft;
  memory_gates<T>(a, b, h, it, ft);
  const float m = fresh ? 0.f : *stm;
  const float m_new = fmaxf(ft + m, it);
  const float keep = expf(ft + m - m_new), add = expf(it - m_new);
  for (int d = tid; d < D; d += 256) {
    ql[d] = Elem<T>::to_f(row[a.q_off + (int64_t)h * D + d]);
    kl[d] = Elem<T>::to_f(row[a.k_off + (int64_t)h * D + d]);
  }
  float av[VEC], y[VEC];
#pragma unroll
  for (int u = 0; u < VEC; ++u) {
    av[u] = e_ok ? add * Elem<T>::to_f(row[a.v_off + (int64_t)h * E + e + u]) : 0.f;
    y[u] = 0.f;
  }
  __syncthreads();
  for (int i0 = 0; 16 * i0 < D; i0 += BATCH) {
    if (i0 > 0) load(i0);
#pragma unroll
    for (int i = 0; i < BATCH; ++i) {
      const int d = rg + 16 * (i0 + i);
      if (d < D) {
        const float kd = kl[d], qd = ql[d];
#pragma unroll
        for (int u = 0; u < VEC; ++u) {
          S[i][u] = keep * S[i][u] + kd * av[u];
          y[u] += S[i][u] * qd;
        }
        if (e_ok) {
          if constexpr (VEC == 4)
            *reinterpret_cast<float4*>(stS + (int64_t)d * E + e) = float4{S[i][0], S[i][1], S[i][2], S[i][3]};
          else
            stS[(int64_t)d * E + e] = S[i][0];
        }
      }
    }
  }
#pragma unroll
  for (int u = 0; u < VEC; ++u) part[rg * COLS + cg * VEC + u] = y[u];
  __syncthreads();
  float* w = a.work + (int64_t)b * a.wld;
  if (tid < COLS && e0 + tid < E) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) s += part[i * COLS + tid];
    w[(int64_t)h * E + e0 + tid] = s * a.q_scale;
  }
  if (lead) {
    float den = 0.f;
    for (int d = tid; d < D; d += 256) {
      const float x = keep * (fresh ? 0.f : stn[d]) + add * kl[d];
      stn[d] = x;
      den += x * ql[d];
    }
    den = block_sum(den, red);
    if (tid == 0) {
      w[(int64_t)H * E + h] = den * a.q_scale;
      w[(int64_t)H * E + H + h] = m_new;        // (the other slices read the old m: memory_keep_max_kernel moves it)
    }
  }
}

// ---------------------------------------------------------------------------------- division, norm, weight, gate
template <typename T, int VEC, bool KEEP_MAX>
__global__ void __launch_bounds__(256) memory_out_kernel(MemArgs a) {
  constexpr int NR = 4;              // pieces of VEC elements a lane keeps (longer heads are read again)
  const int lane = threadIdx.x & 63;
  const int64_t id = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int H = a.H, E = a.E;
  if (id >= a.num_tokens * H) return;
  const int64_t t = id / H;
  const int h = (int)(id % H);
  const float* w = a.work + t * a.wld;
  const float* x = w + (int64_t)h * E;
  const float den = w[(int64_t)H * E + h], m = w[(int64_t)H * E + H + h];
  const float sc = 1.0f / (fmaxf(fabsf(den), expf(-m)) + 1e-6f);
  if (KEEP_MAX && lane == 0 && a.seq_lens[t] > 0)        // one row per request: the running maximum moves into the state here
    a.state[a.state_indices[t] * a.state_ld + (int64_t)H * a.D * E + (int64_t)H * a.D + h] = m;
  const T* g = (const T*)a.p + t * a.ld + a.g_off + (int64_t)h * E;
  const T* nw = (const T*)a.norm_w + (int64_t)h * E;
  T* o = (T*)a.out + t * a.out_ld + (int64_t)h * E;
  float v[NR][VEC], ss = 0.f;
  auto read = [&](int e, float (&f)[VEC]) {
    if constexpr (VEC == 4) {
      const float4 q = *reinterpret_cast<const float4*>(x + e);
      f[0] = q.x * sc; f[1] = q.y * sc; f[2] = q.z * sc; f[3] = q.w * sc;
    } else {
      f[0] = x[e] * sc;
    }
  };
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int e = (i * 64 + lane) * VEC;
#pragma unroll
    for (int u = 0; u < VEC; ++u) v[i][u] = 0.f;
    if (e < E) read(e, v[i]);
#pragma unroll
    for (int u = 0; u < VEC; ++u) ss += v[i][u] * v[i][u];
  }
  for (int e = (NR * 64 + lane) * VEC; e < E; e += 64 * VEC) {
    float f[VEC];
    read(e, f);
#pragma unroll
    for (int u = 0; u < VEC; ++u) ss += f[u] * f[u];
  }
  const float rs = 1.0f / sqrtf(wave_sum(ss) / (float)E + a.eps);
  auto put = [&](int e, const float (&f)[VEC]) {
    T r[VEC];
#pragma unroll
    for (int u = 0; u < VEC; ++u)
      r[u] = Elem<T>::from_f(f[u] * rs * Elem<T>::to_f(nw[e + u]) / (1.0f + expf(-Elem<T>::to_f(g[e + u]))));
    if constexpr (VEC == 4 && sizeof(T) == 2)
      *reinterpret_cast<uint2*>(o + e) = *reinterpret_cast<const uint2*>(r);
    else
#pragma unroll
      for (int u = 0; u < VEC; ++u) o[e + u] = r[u];
  };
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int e = (i * 64 + lane) * VEC;
    if (e < E) put(e, v[i]);
  }
  for (int e = (NR * 64 + lane) * VEC; e < E; e += 64 * VEC) {
    float f[VEC];
    read(e, f);
    put(e, f);
  }
}

}  // namespace semipd

using namespace semipd;

static int64_t memory_row_width(int num_heads, int v_dim) { return ((int64_t)num_heads * v_dim + 2 * num_heads + 3) / 4 * 4; }
extern "C" int64_t semipd_matrix_memory_workspace(int64_t num_tokens, int num_heads, int v_dim) {
  return num_tokens * (memory_row_width(num_heads, v_dim) + kMemPlanes * num_heads);
}
extern "C" int64_t semipd_matrix_memory_state_width(int num_heads, int qk_dim, int v_dim) {
  return (int64_t)num_heads * qk_dim * v_dim + (int64_t)num_heads * qk_dim + num_heads;
}

extern "C" int semipd_matrix_memory(const void* proj, int64_t ld, int64_t q_off, int64_t k_off, int64_t v_off, int64_t g_off,
                                    int64_t i_off, int64_t f_off, const float* i_bias, const float* f_bias, float gate_cap,
                                    const void* norm_w, float eps, float* work, int64_t work_elems, float* state, int64_t state_ld,
                                    const int64_t* state_indices, const int64_t* seq_lens, const int32_t* q_start,
                                    const int32_t* q_len, int64_t batch, int64_t num_tokens, int num_heads, int qk_dim, int v_dim,
                                    float q_scale, void* out, int64_t out_ld, int form, int dtype, void* stream) {
  SEMIPD_CHECK_ARG(batch >= 0 && num_tokens >= 0, SEMIPD_EINVAL, "matrix_memory: bad sizes");
  if (batch == 0 || num_tokens == 0) return 0;
  SEMIPD_CHECK_ARG(num_heads > 0 && qk_dim > 0 && v_dim > 0 && qk_dim <= 1024, SEMIPD_ESHAPE,
                   "matrix_memory: %d heads of %d x %d (keys of at most 1024 elements)", num_heads, qk_dim, v_dim);
  SEMIPD_CHECK_ARG(gate_cap > 0.f, SEMIPD_EINVAL, "matrix_memory: the gates' cap is positive");
  SEMIPD_CHECK_ARG(proj && i_bias && f_bias && norm_w && work && state && state_indices && seq_lens && out, SEMIPD_EINVAL,
                   "matrix_memory: null pointer");
  SEMIPD_CHECK_ARG((q_start == nullptr) == (q_len == nullptr), SEMIPD_EINVAL, "matrix_memory: q_start and q_len come together");
  SEMIPD_CHECK_ARG(q_start != nullptr || num_tokens == batch, SEMIPD_EINVAL, "matrix_memory: one row per request without q_start");
  const int64_t qk = (int64_t)num_heads * qk_dim, vv = (int64_t)num_heads * v_dim;
  SEMIPD_CHECK_ARG(q_off >= 0 && k_off >= 0 && v_off >= 0 && g_off >= 0 && i_off >= 0 && f_off >= 0 && ld >= q_off + qk &&
                       ld >= k_off + qk && ld >= v_off + vv && ld >= g_off + vv && ld >= i_off + num_heads && ld >= f_off + num_heads,
                   SEMIPD_EINVAL, "matrix_memory: a column range leaves the row");
  const int64_t work_ld = memory_row_width(num_heads, v_dim);
  SEMIPD_CHECK_ARG(work_elems >= semipd_matrix_memory_workspace(num_tokens, num_heads, v_dim) && out_ld >= vv &&
                       state_ld >= semipd_matrix_memory_state_width(num_heads, qk_dim, v_dim),
                   SEMIPD_EINVAL, "matrix_memory: rows too short");
  MemArgs a{proj, ld, q_off, k_off, v_off, g_off, i_off, f_off, i_bias, f_bias, gate_cap, work, work_ld, work + num_tokens * work_ld,
            state, state_ld,
            state_indices, seq_lens, q_start, q_len, batch, num_tokens, num_heads, qk_dim, v_dim, q_scale, norm_w, eps, out, out_ld};
  hipStream_t s = as_stream(stream);
  const int64_t esz = dtype == SEMIPD_F32 ? 4 : 2;
  const bool out4 = v_dim % 4 == 0 && work_ld % 4 == 0 && aligned16(work) && ((uintptr_t)out % (4 * esz)) == 0 && out_ld % 4 == 0;
  bool keep_max = false;
  if (q_start == nullptr) {
    const bool vec = v_dim % 4 == 0 && state_ld % 4 == 0 && aligned16(state);
    const int cols = vec ? 64 : 16;
    const size_t bytes = ((size_t)(2 * qk_dim + 3) / 4 * 4 + 16 * (size_t)cols) * sizeof(float);
    const dim3 grid((unsigned)((v_dim + cols - 1) / cols), (unsigned)num_heads, (unsigned)batch);
    SEMIPD_CHECK_ARG(batch <= 65535 && num_heads <= 65535, SEMIPD_ESHAPE, "matrix_memory: too many requests or heads");
    SEMIPD_DISPATCH_DTYPE(dtype, T, {
      if (vec) hipLaunchKernelGGL((memory_step_kernel<T, 4>), grid, dim3(256), bytes, s, a);
      else hipLaunchKernelGGL((memory_step_kernel<T, 1>), grid, dim3(256), bytes, s, a);
    });
    keep_max = true;
  } else {
    const bool chunk_ok = dtype == SEMIPD_BF16 && qk_dim % 8 == 0 && qk_dim <= 256 && v_dim % 8 == 0 && aligned16(proj) && ld % 8 == 0 &&
                          q_off % 8 == 0 && k_off % 8 == 0 && v_off % 8 == 0 && aligned16(work) && ld < (1 << 24);
    SEMIPD_CHECK_ARG(form != 2 || chunk_ok, SEMIPD_ESHAPE, "matrix_memory: the matrix-core form does not take this shape or type");
    if (chunk_ok && form != 1) {
      // (as many chunks as the portions can have: a whole one for every 64 tokens and a short one for every request)
      hipLaunchKernelGGL(memory_gate_kernel, dim3((unsigned)(num_tokens / kMemChunk + batch), (unsigned)((num_heads + 3) / 4)), dim3(256), 0, s, a);
      const int64_t items = batch * num_heads * ((v_dim + kMemCols - 1) / kMemCols);
      const dim3 grid((unsigned)((items + 7) / 8 * 8));
      static std::atomic<uint64_t> done[3] = {};
#define SEMIPD_MEM_CHUNK(ND, SLOT)                                                                                             \
  do {                                                                                                                        \
    constexpr size_t bytes = mem_chunk_lds<ND>();                                                                             \
    if (bytes > 65536 && ensure_dynamic_lds((const void*)memory_chunk_kernel<ND>, bytes, done[SLOT], "matrix_memory"))        \
      return SEMIPD_EINVAL;                                                                                                   \
    hipLaunchKernelGGL((memory_chunk_kernel<ND>), grid, dim3(256), bytes, s, a);                                              \
  } while (0)
      if (qk_dim <= 64) SEMIPD_MEM_CHUNK(2, 0);
      else if (qk_dim <= 128) SEMIPD_MEM_CHUNK(4, 1);
      else SEMIPD_MEM_CHUNK(8, 2);
#undef SEMIPD_MEM_CHUNK
    } else {
#define SEMIPD_MEM_SCAN(NPT, NS, STAGE)                                                                                        \
  do {                                                                                                                        \
    constexpr int cols = 64 / NS;                                                                                             \
    const unsigned blocks = (unsigned)(batch * num_heads * ((v_dim + 1 + cols - 1) / cols));                                  \
    const size_t bytes = (size_t)STAGE * (2 * NPT * NS + cols) * sizeof(float);                                               \
    SEMIPD_DISPATCH_DTYPE(dtype, T,                                                                                           \
                          hipLaunchKernelGGL((memory_scan_kernel<T, NPT, NS>), dim3(blocks), dim3(64), bytes, s, a, STAGE));   \
  } while (0)
      if (qk_dim <= 32) SEMIPD_MEM_SCAN(32, 1, 8);
      else if (qk_dim <= 64) SEMIPD_MEM_SCAN(32, 2, 8);
      else if (qk_dim <= 128) SEMIPD_MEM_SCAN(32, 4, 8);
      else if (qk_dim <= 256) SEMIPD_MEM_SCAN(32, 8, 8);
      else if (qk_dim <= 512) SEMIPD_MEM_SCAN(32, 16, 8);
      else SEMIPD_MEM_SCAN(64, 16, 4);
#undef SEMIPD_MEM_SCAN
    }
    hipLaunchKernelGGL(memory_keep_max_kernel, dim3((unsigned)((batch * num_heads + 63) / 64)), dim3(64), 0, s, a);
  }
  const dim3 ogrid((unsigned)((num_tokens * num_heads + 3) / 4));
  SEMIPD_DISPATCH_DTYPE(dtype, T, {
    if (out4 && keep_max) hipLaunchKernelGGL((memory_out_kernel<T, 4, true>), ogrid, dim3(256), 0, s, a);
    else if (out4) hipLaunchKernelGGL((memory_out_kernel<T, 4, false>), ogrid, dim3(256), 0, s, a);
    else if (keep_max) hipLaunchKernelGGL((memory_out_kernel<T, 1, true>), ogrid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((memory_out_kernel<T, 1, false>), ogrid, dim3(256), 0, s, a);
  });
  return launch_status("matrix_memory");
}
