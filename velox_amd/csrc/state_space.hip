// Kernels of the selective state space mixer for gfx950.  Per sequence and head, with step size d = softplus(dt + dt_bias), input x
// (vdim channels) and vectors B, C (N entries, shared by the heads of a group), from the state S (N x vdim float32) of the slot:
//   S <- exp(-rate d) S + d B x^T;   y = S^T C + skip x.
//   state_space_step      token by token: single tokens and short portions, every size
//   state_space_chunk     long portions in chunks of 64 tokens on v_mfma_f32_16x16x4_f32, three kernels (see below)
//   gated_group_norm      y silu(z), normed in equal parts of a row, times a weight
// A row of `xbc` holds [x: heads * vdim | B: groups * N | C: groups * N], float32 or bfloat16; dt stands in another tensor's row.
// Everything between a load and a store is float32 (sums of a chunk's log-decays float64).  No result depends on what else
// is in the batch.
#include "common.h"

__device__ __forceinline__ float softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

struct StateSpaceArgs {
  const void* xbc;
  int ld;                 // elements per row of xbc
  const void* step_src;   // same type as xbc
  int step_ld, step_at;
  const float* dt_bias;
  const float* rate;
  const float* skip;
  float* state;           // [slots, heads, N, vdim]
  const int* slots;
  const int* cu_q;
  float* out;             // [T, heads * vdim]
  int heads, groups, N, vdim;
  float* local;           // chunks: [chunk slots, heads, N, vdim]
  float* carry;           // chunks: [chunk slots, heads]
};

template <typename T> __device__ __forceinline__ float step_size(const StateSpaceArgs& a, size_t t, int h) {
  return softplus(to_f32(((const T*)a.step_src)[t * a.step_ld + a.step_at + h]) + a.dt_bias[h]);
}

// ---------------------------------------------------------------------------------------------
// state_space_step.  Grid (tiles of CW columns, heads, sequences), 256 lanes: lane = (row group, column); a lane holds the rows
// row_group + i * (256 / CW), i < NR, of its column in registers through the whole portion.  A token's B and C wait in LDS (two
// buffers); its read-out is summed over a wave's row groups by exchanges and over the waves through LDS.  CW and NR
// follow from the sizes alone, and so does the order of every sum.
// ---------------------------------------------------------------------------------------------
template <typename T, int CW, int NR>
__global__ void __launch_bounds__(256) state_space_step_kernel(const StateSpaceArgs a) {
  constexpr int RG = 256 / CW;
  extern __shared__ float bc[];  // [2][2 * N]
  __shared__ float part[2][4][CW];
  const int tid = threadIdx.x, col = tid % CW, rg = tid / CW, wave = tid >> 6;
  const int h = blockIdx.y, b = blockIdx.z;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  if (hi <= lo) return;  // (the whole workgroup)
  const int N = a.N, vdim = a.vdim, inner = a.heads * vdim;
  const int v = blockIdx.x * CW + col;
  const bool live = v < vdim;
  const int vc = live ? v : vdim - 1;  // (lanes beyond the last column follow it and write nothing)
  const int g = h / (a.heads / a.groups);
  const float rate = a.rate[h], skip = a.skip[h];
  const T* rows = (const T*)a.xbc;
  const int b_at = inner + g * N, c_at = inner + a.groups * N + g * N;
  float* S = a.state + (((size_t)a.slots[b] * a.heads + h) * N) * vdim + vc;
  float s[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const int n = rg + i * RG;
    s[i] = n < N ? S[(size_t)n * vdim] : 0.f;
  }
  auto stage = [&](int t, int buffer) {
    const T* row = rows + (size_t)t * a.ld;
    float* to = bc + buffer * 2 * N;
    for (int n = tid; n < N; n += 256) {
      to[n] = to_f32(row[b_at + n]);
      to[N + n] = to_f32(row[c_at + n]);
    }
  };
  stage(lo, 0);
  float x = to_f32(rows[(size_t)lo * a.ld + h * vdim + vc]);
  float d = step_size<T>(a, lo, h);
  __syncthreads();
  for (int t = lo; t < hi; ++t) {
    const int buffer = (t - lo) & 1;
    float next_x = 0.f, next_d = 0.f;
    if (t + 1 < hi) {
      stage(t + 1, buffer ^ 1);
      next_x = to_f32(rows[(size_t)(t + 1) * a.ld + h * vdim + vc]);
      next_d = step_size<T>(a, t + 1, h);
    }
    const float decay = expf(-rate * d), write = d * x;
    const float* from = bc + buffer * 2 * N;
    float y = 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int n = rg + i * RG;
      if (n < N) {
        s[i] = s[i] * decay + from[n] * write;
        y += s[i] * from[N + n];
      }
    }
#pragma unroll
    for (int off = CW; off < 64; off <<= 1) y += __shfl_xor(y, off, VELOX_WAVE);
    if ((tid & 63) < CW) part[buffer][wave][col] = y;
    __syncthreads();  // (also: the next token's B and C are in place, and everyone is done with this token's)
    if (tid < CW && live)
      a.out[(size_t)t * inner + h * vdim + v] = ((part[buffer][0][col] + part[buffer][1][col]) + (part[buffer][2][col] + part[buffer][3][col])) + skip * x;
    x = next_x;
    d = next_d;
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int n = rg + i * RG;
      if (n < N) S[(size_t)n * vdim] = s[i];
    }
  }
}

// ---------------------------------------------------------------------------------------------
// Long portions.  A sequence's portion is cut into chunks of Q = 64 tokens.  With A_t the running sum of the log-decays -rate d
// inside a chunk (inclusive), A_Q its total, and Z the state before the chunk:
//   y_t = exp(A_t) Z^T C_t + sum_{s <= t} exp(A_t - A_s) d_s (B_s . C_t) x_s + skip x_t
//   S'  = exp(A_Q) Z + sum_s exp(A_Q - A_s) d_s B_s x_s^T
// state_space_local_kernel   the second sum of S' for every chunk at once (and exp(A_Q))
// state_space_chain_kernel   the only dependent chain: Z of every chunk, element by element, in the place of the sums
// state_space_output_kernel  y of every chunk at once
// Every exponent is a difference of sums that is at most 0; the sums are float64, so a difference of two large ones is as
// exact as a small one.  Sequence b's chunk c has the scratch slot cu_q[b] / 64 + b + c: no two chunks share one, and
// there are fewer than T / 64 + sequences.
// Operands of v_mfma_f32_16x16x4_f32: lane (g, i) = (lane / 16, lane % 16) gives row i of the left and column i of the right matrix
// at inner index g; the result holds rows 4 g .. 4 g + 3 of column i.  The inner index may be taken in any order, so four
// instructions take the 16 indices 4 g + r, r = 0 .. 3, one r each.
// ---------------------------------------------------------------------------------------------
#define SS_CHUNK 64
#define SS_ROWS 128  // entries of B (rows of the state) a workgroup works on at a time
#define SS_COLS 64   // columns of the state a workgroup works on
#define SS_HALF 32   // tokens of a chunk that state_space_local_kernel holds in LDS at a time
#define SS_LOCAL_B (SS_ROWS + 16)  // LDS row strides: 16 (mod 64) for reads of four rows x 16 neighbours,
#define SS_LOCAL_X (SS_COLS + 16)
#define SS_SLICE 32  // entries of B and C the read-out takes at a time
#define SS_OUT_B (SS_SLICE + 4)    // 4 (mod 32) for 16 rows x 16 bytes, and for every fourth row x 16 neighbours
#define SS_OUT_X (SS_COLS + 4)

__device__ __forceinline__ float4_t mma4(float a, float b, float4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }

// step sizes and running sums of the log-decays of a chunk's tokens (tokens beyond `count`: step 0, no decay); wave 0 works
template <typename T>
__device__ __forceinline__ void chunk_steps(const StateSpaceArgs& a, int t0, int count, int h, float* steps, double* sums) {
  if (threadIdx.x < 64) {
    const int lane = threadIdx.x;
    const float d = lane < count ? step_size<T>(a, (size_t)t0 + lane, h) : 0.f;
    double total = -(double)(a.rate[h] * d);
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const double before = __shfl_up(total, off, VELOX_WAVE);
      if (lane >= off) total += before;
    }
    steps[lane] = d;
    sums[lane] = total;
  }
}

// ROWS rows of COLS columns from `from` on (`ld` elements apart) into LDS rows of `stride` floats: the first `count` rows and `width`
// columns are there, the others become zeros.  In two halves, so that a lane's loads are all under way before one is waited for
// (load) and something else can stand between them and the stores (store).
template <typename T, int ROWS, int COLS>
struct StagedRows {
  static constexpr int QUADS = COLS / 4, EACH = ROWS * QUADS / 256;
  static_assert(ROWS * QUADS % 256 == 0, "every lane carries the same number of pieces");
  float v[EACH][4];
  __device__ __forceinline__ void load(const T* from, int ld, int count, int width, bool vec) {
    if (vec) {  // (widths are multiples of four, and so is every row's start)
#pragma unroll
      for (int e = 0; e < EACH; ++e) {
        const int index = threadIdx.x + e * 256, r = index / QUADS, c = index % QUADS * 4;
        // (a piece that is not there is read from the first row and then cleared: no branch around the load)
        const bool there = r < count && c < width;
        const T* p = there ? from + (size_t)r * ld + c : from;
        if constexpr (sizeof(T) == 4) {
          const float4_t x = *reinterpret_cast<const float4_t*>(p);
#pragma unroll
          for (int j = 0; j < 4; ++j) v[e][j] = there ? x[j] : 0.f;
        } else {
          const short4_t x = *reinterpret_cast<const short4_t*>(p);
#pragma unroll
          for (int j = 0; j < 4; ++j) v[e][j] = there ? __uint_as_float(((uint32_t)(uint16_t)x[j]) << 16) : 0.f;
        }
      }
    } else {
#pragma unroll
      for (int e = 0; e < EACH; ++e) {
        const int index = threadIdx.x + e * 256, r = index / QUADS, c = index % QUADS * 4;
        load4<T>(from, (size_t)r * ld, c, width, r < count, false, v[e]);
      }
    }
  }
  __device__ __forceinline__ void store(float* to, int stride) const {
#pragma unroll
    for (int e = 0; e < EACH; ++e) {
      const int index = threadIdx.x + e * 256, r = index / QUADS, c = index % QUADS * 4;
      *reinterpret_cast<float4_t*>(to + r * stride + c) = float4_t{v[e][0], v[e][1], v[e][2], v[e][3]};
    }
  }
};

template <typename T>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(4, 8))) state_space_local_kernel(const StateSpaceArgs a, int row_slices, int col_slices, int vec) {
  __shared__ __attribute__((aligned(16))) float bs[SS_HALF * SS_LOCAL_B];  // half of the chunk's tokens at a time
  __shared__ __attribute__((aligned(16))) float xs[SS_HALF * SS_LOCAL_X];
  __shared__ float steps[64];
  __shared__ double sums[64];
  const int h = blockIdx.y, b = blockIdx.z;
  int chunk = blockIdx.x;
  const int cs = chunk % col_slices; chunk /= col_slices;
  const int rs = chunk % row_slices; chunk /= row_slices;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  const int t0 = lo + chunk * SS_CHUNK;
  if (t0 >= hi) return;  // (the whole workgroup)
  const int count = hi - t0 < SS_CHUNK ? hi - t0 : SS_CHUNK;
  const int N = a.N, vdim = a.vdim, inner = a.heads * vdim;
  const int g = h / (a.heads / a.groups);
  const T* rows = (const T*)a.xbc;
  const int n0 = rs * SS_ROWS, v0 = cs * SS_COLS;
  const int n_width = N - n0 < SS_ROWS ? N - n0 : SS_ROWS, v_width = vdim - v0 < SS_COLS ? vdim - v0 : SS_COLS;
  const int n_tiles = (n_width + 15) / 16, v_tiles = (v_width + 15) / 16;
  StagedRows<T, SS_HALF, SS_ROWS> b_rows;
  StagedRows<T, SS_HALF, SS_COLS> x_rows;
  auto load_half = [&](int half) {
    const int first = half * SS_HALF, here = count > first ? count - first : 0;
    const T* from = rows + (size_t)(t0 + (here > 0 ? first : 0)) * a.ld;
    x_rows.load(from + h * vdim + v0, a.ld, here, v_width, vec);
    b_rows.load(from + inner + g * N + n0, a.ld, here, n_width, vec);
  };
  load_half(0);
  chunk_steps<T>(a, t0, count, h, steps, sums);
  __syncthreads();
  const double end = sums[63];
  const size_t slot = (size_t)(lo / SS_CHUNK) + b + chunk;
  if (threadIdx.x == 0 && rs == 0 && cs == 0) a.carry[slot * a.heads + h] = expf((float)end);
  if (threadIdx.x < 64) steps[threadIdx.x] *= expf((float)(end - sums[threadIdx.x]));  // what x_s is multiplied by
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int gg = lane >> 4, i = lane & 15;
  float* local = a.local + (slot * a.heads + h) * (size_t)N * vdim;
  // a wave takes a pair of row tiles, all column tiles (four at most)
  const int nt = 2 * wave;
  const bool first = nt < n_tiles, second = nt + 1 < n_tiles;
  float4_t acc[2][4];
#pragma unroll
  for (int p = 0; p < 2; ++p)
#pragma unroll
    for (int c = 0; c < 4; ++c) acc[p][c] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int half = 0; half < SS_CHUNK / SS_HALF; ++half) {
    __syncthreads();  // (the factors are in place; later: everyone is done with the half before)
    b_rows.store(bs, SS_LOCAL_B);
#pragma unroll
    for (int e = 0; e < x_rows.EACH; ++e) {
      const float factor = steps[half * SS_HALF + (threadIdx.x + e * 256) / x_rows.QUADS];
#pragma unroll
      for (int j = 0; j < 4; ++j) x_rows.v[e][j] *= factor;
    }
    x_rows.store(xs, SS_LOCAL_X);
    __syncthreads();
    if (half + 1 < SS_CHUNK / SS_HALF) load_half(half + 1);  // (in flight while this half is worked)
    if (first) {
      const float* b0 = bs + gg * SS_LOCAL_B + nt * 16 + i;
      const float* b1 = b0 + (second ? 16 : 0);
      const float* x0 = xs + gg * SS_LOCAL_X + i;
#pragma unroll
      for (int k = 0; k < SS_HALF / 4; ++k) {
        const float first_row = b0[k * 4 * SS_LOCAL_B], second_row = b1[k * 4 * SS_LOCAL_B];
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          if (c < v_tiles) {
            const float xv = x0[k * 4 * SS_LOCAL_X + 16 * c];
            acc[0][c] = mma4(first_row, xv, acc[0][c]);
            acc[1][c] = mma4(second_row, xv, acc[1][c]);
          }
        }
      }
    }
  }
  if (first) {
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      if (p == 1 && !second) break;
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        if (c >= v_tiles) break;
        const int v = v0 + 16 * c + i;
        if (v >= vdim) continue;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int n = n0 + (nt + p) * 16 + 4 * gg + j;
          if (n < N) local[(size_t)n * vdim + v] = acc[p][c][j];
        }
      }
    }
  }
}

// One element (or piece of four) of a head's state per lane: Z of every chunk takes the place of the chunk's own sum.
template <typename P>
__global__ void __launch_bounds__(256) state_space_chain_kernel(const StateSpaceArgs a, int pieces) {
  const int e = blockIdx.x * 256 + threadIdx.x;
  const int h = blockIdx.y, b = blockIdx.z;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  if (e >= pieces || hi <= lo) return;
  const int chunks = (hi - lo + SS_CHUNK - 1) / SS_CHUNK;
  const size_t first = (size_t)(lo / SS_CHUNK) + b;
  P* state = reinterpret_cast<P*>(a.state) + ((size_t)a.slots[b] * a.heads + h) * pieces + e;
  P* at = reinterpret_cast<P*>(a.local) + (first * a.heads + h) * pieces + e;
  const size_t stride = (size_t)a.heads * pieces;
  const float* carry = a.carry + first * a.heads + h;
  P z = *state;
  constexpr int AHEAD = 8;  // sums asked for together
  for (int c0 = 0; c0 < chunks; c0 += AHEAD) {
    P held[AHEAD];
    float f[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      const int c = c0 + j < chunks ? c0 + j : chunks - 1;
      held[j] = at[c * stride];
      f[j] = carry[(size_t)c * a.heads];
    }
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
      if (c0 + j < chunks) {
        at[(c0 + j) * stride] = z;
        z = z * f[j] + held[j];
      }
    }
  }
  *state = z;
}

template <typename T>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(4, 4))) state_space_output_kernel(const StateSpaceArgs a, int col_slices, int vec) {
  __shared__ __attribute__((aligned(16))) float bs[SS_CHUNK * SS_OUT_B];  // a slice of B's columns, of Z's rows
  __shared__ __attribute__((aligned(16))) float zs[SS_SLICE * SS_OUT_X];
  __shared__ __attribute__((aligned(16))) float xs[SS_CHUNK * SS_OUT_X];
  __shared__ float steps[64];
  __shared__ double sums[64];
  const int h = blockIdx.y, b = blockIdx.z;
  const int cs = blockIdx.x % col_slices, chunk = blockIdx.x / col_slices;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  const int t0 = lo + chunk * SS_CHUNK;
  if (t0 >= hi) return;  // (the whole workgroup)
  const int count = hi - t0 < SS_CHUNK ? hi - t0 : SS_CHUNK;
  const int N = a.N, vdim = a.vdim, inner = a.heads * vdim;
  const int g = h / (a.heads / a.groups);
  const T* rows = (const T*)a.xbc;
  const int v0 = cs * SS_COLS;
  const int v_width = vdim - v0 < SS_COLS ? vdim - v0 : SS_COLS, v_tiles = (v_width + 15) / 16;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int gg = lane >> 4, i = lane & 15;
  const int my_row = wave * 16 + i;  // the token of the chunk whose read-out this lane's column is
  const bool row_ok = my_row < count;
  const bool busy = wave * 16 < count;  // (the same for the whole wave)
  const T* chunk_rows = rows + (size_t)t0 * a.ld;
  const T* c_row = chunk_rows + (size_t)(row_ok ? my_row : 0) * a.ld + inner + a.groups * N + g * N;
  const size_t slot = (size_t)(lo / SS_CHUNK) + b + chunk;
  const float* Z = a.local + (slot * a.heads + h) * (size_t)N * vdim;
  const bool z_vec = vdim % 4 == 0;
  float4_t scores[4], acc[4];  // (B_s . C_t) of the four tiles of s; the read-out's four column tiles
#pragma unroll
  for (int c = 0; c < 4; ++c) scores[c] = acc[c] = float4_t{0.f, 0.f, 0.f, 0.f};
  StagedRows<T, SS_CHUNK, SS_COLS> x_rows;
  StagedRows<T, SS_CHUNK, SS_SLICE> b_rows;
  StagedRows<float, SS_SLICE, SS_COLS> z_rows;
  float c_held[SS_SLICE / 16][4];  // this lane's entries of C_t: 16 kb + 4 gg .. + 3 of the slice
  auto load_slice = [&](int n0) {
    const int n_width = N - n0 < SS_SLICE ? N - n0 : SS_SLICE;
    b_rows.load(chunk_rows + inner + g * N + n0, a.ld, count, n_width, vec);
    z_rows.load(Z + (size_t)n0 * vdim + v0, vdim, n_width, v_width, z_vec);
#pragma unroll
    for (int kb = 0; kb < SS_SLICE / 16; ++kb) {
      if (vec) {
        const bool there = row_ok && 16 * kb + 4 * gg < n_width;
        float x[4];
        load4<T>(there ? c_row + n0 + 16 * kb + 4 * gg : c_row, 0, 0, 4, true, true, x);
#pragma unroll
        for (int j = 0; j < 4; ++j) c_held[kb][j] = there ? x[j] : 0.f;
      } else {
        load4<T>(c_row + n0, 0, 16 * kb + 4 * gg, n_width, row_ok, false, c_held[kb]);
      }
    }
  };
  x_rows.load(chunk_rows + h * vdim + v0, a.ld, count, v_width, vec);
  load_slice(0);
  chunk_steps<T>(a, t0, count, h, steps, sums);
  x_rows.store(xs, SS_OUT_X);
  for (int n0 = 0; n0 < N; n0 += SS_SLICE) {
    b_rows.store(bs, SS_OUT_B);
    z_rows.store(zs, SS_OUT_X);
    __syncthreads();
    float c_now[SS_SLICE / 16][4];
#pragma unroll
    for (int kb = 0; kb < SS_SLICE / 16; ++kb)
#pragma unroll
      for (int j = 0; j < 4; ++j) c_now[kb][j] = c_held[kb][j];
    if (n0 + SS_SLICE < N) load_slice(n0 + SS_SLICE);  // (in flight while this slice is worked)
    if (busy) {
#pragma unroll
      for (int kb = 0; kb < SS_SLICE / 16; ++kb) {
#pragma unroll
        for (int t = 0; t < 4; ++t) {
          if (t > wave) continue;  // (tokens behind this wave's)
          const float4_t bv = *reinterpret_cast<const float4_t*>(bs + (16 * t + i) * SS_OUT_B + 16 * kb + 4 * gg);
#pragma unroll
          for (int r = 0; r < 4; ++r) scores[t] = mma4(bv[r], c_now[kb][r], scores[t]);
        }
        const float* z0 = zs + (16 * kb + 4 * gg) * SS_OUT_X + i;
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int c = 0; c < 4; ++c)
            if (c < v_tiles) acc[c] = mma4(z0[r * SS_OUT_X + 16 * c], c_now[kb][r], acc[c]);
      }
    }
    __syncthreads();  // everyone is done with the slice
  }
  if (!busy) return;  // (no barrier follows)
  const double mine = sums[my_row];
  const float before = expf((float)mine);
#pragma unroll
  for (int c = 0; c < 4; ++c) acc[c] = acc[c] * before;
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    if (t > wave) continue;
    float m[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int s = 16 * t + 4 * gg + r;
      m[r] = s <= my_row ? scores[t][r] * (expf((float)(mine - sums[s])) * steps[s]) : 0.f;
    }
    const float* x0 = xs + (16 * t + 4 * gg) * SS_OUT_X + i;
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int c = 0; c < 4; ++c)
        if (c < v_tiles) acc[c] = mma4(x0[r * SS_OUT_X + 16 * c], m[r], acc[c]);
  }
  if (!row_ok) return;
  const float skip = a.skip[h];
  float* out = a.out + (size_t)(t0 + my_row) * inner + h * vdim + v0;
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    if (c >= v_tiles) break;
    const float4_t x = *reinterpret_cast<const float4_t*>(xs + my_row * SS_OUT_X + 16 * c + 4 * gg);
    const float4_t y = acc[c] + x * skip;
    const int v = 16 * c + 4 * gg;
    if (z_vec && v + 4 <= v_width) *reinterpret_cast<float4_t*>(out + v) = y;
    else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (v + j < v_width) out[v + j] = y[j];
    }
  }
}

// Largest state the token-by-token kernel holds in registers.
extern "C" int velox_state_space_max_state() { return 1024; }

// float32 elements of scratch that chunks need
extern "C" long long velox_state_space_scratch_elems(int tokens, int num_seqs, int heads, int N, int vdim) {
  const long long slots = tokens / SS_CHUNK + num_seqs;
  return slots * heads * ((long long)N * vdim + 1) + 4;
}

template <typename T, int CW>
static int launch_step(const StateSpaceArgs& a, int num_seqs, hipStream_t stream) {
  const dim3 grid((a.vdim + CW - 1) / CW, a.heads, num_seqs);
  const size_t lds = (size_t)4 * a.N * sizeof(float);
  const int per_lane = (a.N + 256 / CW - 1) / (256 / CW);
  if (per_lane <= 4) state_space_step_kernel<T, CW, 4><<<grid, 256, lds, stream>>>(a);
  else if (per_lane <= 8) state_space_step_kernel<T, CW, 8><<<grid, 256, lds, stream>>>(a);
  else if (per_lane <= 16) state_space_step_kernel<T, CW, 16><<<grid, 256, lds, stream>>>(a);
  else if (per_lane <= 32) state_space_step_kernel<T, CW, 32><<<grid, 256, lds, stream>>>(a);
  else return (int)hipErrorInvalidValue;
  return (int)hipGetLastError();
}

template <typename T>
static int launch_state_space(StateSpaceArgs a, float* scratch, int tokens, int num_seqs, int max_q_len, hipStream_t stream) {
  if (scratch == nullptr) {
    if (a.N > 512) return launch_step<T, 8>(a, num_seqs, stream);
    if (a.N > 256 || a.vdim <= 16) return launch_step<T, 16>(a, num_seqs, stream);
    return launch_step<T, 32>(a, num_seqs, stream);
  }
  const long long slots = tokens / SS_CHUNK + num_seqs;
  a.local = scratch;
  a.carry = scratch + slots * a.heads * a.N * a.vdim;
  const int chunks = (max_q_len + SS_CHUNK - 1) / SS_CHUNK;
  const int row_slices = (a.N + SS_ROWS - 1) / SS_ROWS, col_slices = (a.vdim + SS_COLS - 1) / SS_COLS;
  // pieces of four neighbours of a row of xbc can be read whole
  const int vec = a.ld % 4 == 0 && a.vdim % 4 == 0 && a.N % 4 == 0 && (uintptr_t)a.xbc % (4 * sizeof(T)) == 0;
  state_space_local_kernel<T><<<dim3((unsigned)chunks * row_slices * col_slices, a.heads, num_seqs), 256, 0, stream>>>(a, row_slices, col_slices, vec);
  const int elems = a.N * a.vdim;
  if (elems % 4 == 0 && (((uintptr_t)a.state | (uintptr_t)scratch) & 15) == 0)
    state_space_chain_kernel<float4_t><<<dim3((elems / 4 + 255) / 256, a.heads, num_seqs), 256, 0, stream>>>(a, elems / 4);
  else
    state_space_chain_kernel<float><<<dim3((elems + 255) / 256, a.heads, num_seqs), 256, 0, stream>>>(a, elems);
  state_space_output_kernel<T><<<dim3((unsigned)chunks * col_slices, a.heads, num_seqs), 256, 0, stream>>>(a, col_slices, vec);
  return (int)hipGetLastError();
}

// scratch: nullptr (token by token), or velox_state_space_scratch_elems float32 (chunks)
extern "C" int velox_state_space_scan(const void* xbc, int dtype, int ld, const void* step_src, int step_ld, int step_at, const float* dt_bias, const float* rate,
                                      const float* skip, float* state, const int* slots, const int* cu_q, float* out, float* scratch, int tokens, int num_seqs,
                                      int max_q_len, int heads, int groups, int N, int vdim, hipStream_t stream) {
  if (tokens <= 0 || num_seqs <= 0) return 0;
  if (heads < 1 || groups < 1 || heads % groups != 0 || N < 1 || N > 1024 || vdim < 1 || heads > 65535 || num_seqs > 65535 || max_q_len < 1)
    return (int)hipErrorInvalidValue;
  StateSpaceArgs a{xbc, ld, step_src, step_ld, step_at, dt_bias, rate, skip, state, slots, cu_q, out, heads, groups, N, vdim, nullptr, nullptr};
  if (dtype == VELOX_BF16) return launch_state_space<bf16_t>(a, scratch, tokens, num_seqs, max_q_len, stream);
  return launch_state_space<float>(a, scratch, tokens, num_seqs, max_q_len, stream);
}

// ---------------------------------------------------------------------------------------------
// gated_group_norm: one workgroup per token and part of a row (part = width / groups): y = read * silu(z), out = y / sqrt(mean(y^2) + eps)
// over the part, times weight.  z stands in a token's row of gate_src at gate_at.  Parts of a multiple of four lie in registers
// as pieces of four (PIECES per lane); others are worked element by element, twice.
// ---------------------------------------------------------------------------------------------
struct GroupNormArgs {
  const float* read;
  const void* gate;
  int gate_bf16, gate_ld, gate_at;
  const float* weight;
  void* out;
  int out_bf16, width, part;
  float eps;
};

__device__ __forceinline__ float silu_of(float z) { return z / (1.f + expf(-z)); }

template <int PIECES>
__global__ void __launch_bounds__(256) gated_group_norm_vec_kernel(const GroupNormArgs a) {
  __shared__ float scratch[16];
  const size_t row = (size_t)blockIdx.x * a.width;
  const size_t gate_row = (size_t)blockIdx.x * a.gate_ld + a.gate_at;
  const int first = blockIdx.y * a.part;
  float4_t held[PIECES];
  float sumsq = 0.f;
#pragma unroll
  for (int p = 0; p < PIECES; ++p) {
    const int at = (threadIdx.x + p * blockDim.x) * 4;
    held[p] = float4_t{0.f, 0.f, 0.f, 0.f};
    if (at < a.part) {
      const float4_t y = *reinterpret_cast<const float4_t*>(a.read + row + first + at);
      float4_t z;
      if (a.gate_bf16) {
        const short4_t raw = *reinterpret_cast<const short4_t*>((const bf16_t*)a.gate + gate_row + first + at);
#pragma unroll
        for (int j = 0; j < 4; ++j) z[j] = __uint_as_float(((uint32_t)(uint16_t)raw[j]) << 16);
      } else {
        z = *reinterpret_cast<const float4_t*>((const float*)a.gate + gate_row + first + at);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        held[p][j] = y[j] * silu_of(z[j]);
        sumsq += held[p][j] * held[p][j];
      }
    }
  }
  const float inv = 1.f / sqrtf(block_sum(sumsq, scratch) / (float)a.part + a.eps);
#pragma unroll
  for (int p = 0; p < PIECES; ++p) {
    const int at = (threadIdx.x + p * blockDim.x) * 4;
    if (at < a.part) {
      const float4_t o = held[p] * inv * *reinterpret_cast<const float4_t*>(a.weight + first + at);
      if (a.out_bf16) {
        short4_t bits;
#pragma unroll
        for (int j = 0; j < 4; ++j) bits[j] = bf16_bits(o[j]);
        *reinterpret_cast<short4_t*>((bf16_t*)a.out + row + first + at) = bits;
      } else {
        *reinterpret_cast<float4_t*>((float*)a.out + row + first + at) = o;
      }
    }
  }
}

__global__ void __launch_bounds__(256) gated_group_norm_kernel(const GroupNormArgs a) {
  __shared__ float scratch[16];
  const size_t row = (size_t)blockIdx.x * a.width;
  const size_t gate_row = (size_t)blockIdx.x * a.gate_ld + a.gate_at;
  const int first = blockIdx.y * a.part;
  auto value = [&](int i) {
    const float z = a.gate_bf16 ? to_f32(((const bf16_t*)a.gate)[gate_row + i]) : ((const float*)a.gate)[gate_row + i];
    return a.read[row + i] * silu_of(z);
  };
  float sumsq = 0.f;
  for (int i = first + threadIdx.x; i < first + a.part; i += 256) { const float y = value(i); sumsq += y * y; }
  const float inv = 1.f / sqrtf(block_sum(sumsq, scratch) / (float)a.part + a.eps);
  for (int i = first + threadIdx.x; i < first + a.part; i += 256) {
    const float o = value(i) * inv * a.weight[i];
    if (a.out_bf16) ((bf16_t*)a.out)[row + i] = (bf16_t)o;
    else ((float*)a.out)[row + i] = o;
  }
}

extern "C" int velox_gated_group_norm(const float* read, const void* gate, int gate_dtype, int gate_ld, int gate_at, const float* weight, float eps, void* out,
                                      int out_dtype, int tokens, int width, int groups, hipStream_t stream) {
  if (tokens <= 0) return 0;
  if (groups < 1 || groups > 65535 || width % groups != 0) return (int)hipErrorInvalidValue;
  GroupNormArgs a{read, gate, gate_dtype == VELOX_BF16, gate_ld, gate_at, weight, out, out_dtype == VELOX_BF16, width, width / groups, eps};
  const dim3 grid(tokens, groups);
  const size_t gate_elem = a.gate_bf16 ? 2 : 4;
  const bool aligned = a.part % 4 == 0 && gate_ld % 4 == 0 && gate_at % 4 == 0 && (((uintptr_t)read | (uintptr_t)weight | (uintptr_t)out) & 15) == 0 &&
                       (uintptr_t)gate % (4 * gate_elem) == 0;
  const int pieces = a.part / 4;
  int lanes = (pieces + 63) / 64 * 64;
  lanes = lanes < 64 ? 64 : lanes > 256 ? 256 : lanes;
  const int per_lane = (pieces + lanes - 1) / lanes;
  if (!aligned || per_lane > 16) gated_group_norm_kernel<<<grid, 256, 0, stream>>>(a);
  else if (per_lane <= 1) gated_group_norm_vec_kernel<1><<<grid, lanes, 0, stream>>>(a);
  else if (per_lane <= 4) gated_group_norm_vec_kernel<4><<<grid, lanes, 0, stream>>>(a);
  else gated_group_norm_vec_kernel<16><<<grid, lanes, 0, stream>>>(a);
  VELOX_RETURN_LAUNCH_STATUS();
}
