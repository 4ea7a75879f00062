// The generalized delta rule over long portions of prompts, in chunks of 16 tokens on the float32 matrix instructions.
//
// Per head, with decay w_t, unit key u_t, removal vector b_t = a_t * u_t, key k_t, value v_t and read vector r_t:
//     S_t = diag(w_t) S_(t-1) - b_t (u_t^T S_(t-1)) + k_t v_t^T,   o_t = S_t^T r_t.
// Inside a chunk let P_t = w_1 * .. * w_t (per channel, P_0 = 1) and S_t = diag(P_t) Z_t.  With
//     U_t = u_t * P_(t-1),  R_t = r_t * P_t,  B_t = b_t / P_t,  K_t = k_t / P_t       (rows of 16 x dim matrices)
// the rule reads Z_t = Z_(t-1) - B_t d_t + K_t v_t^T with the removed rows d_t = U_t Z_(t-1), so that
//     D = U Z_0 + M1 V - M2 D,   O = R Z_0 + M3 V - M4 D,   Z_16 = Z_0 + K^T V - B^T D,
// M1 = U K^T and M2 = U B^T below the diagonal, M3 = R K^T and M4 = R B^T with it.  With T = (I + M2)^-1 (unit lower
// triangular, by substitution) everything that does not touch the state is worked for all chunks at the same time:
//     U' = T U,   Dv = T M1 V,   R' = R - M4 T U,   Ov = M3 V - M4 Dv,
// and what is left of the dependent chain is, per chunk,   D = U' Z_0 + Dv,   O = R' Z_0 + Ov,   S = diag(P_16) (Z_0 + K^T V - B^T D).
// All of it is float32.  A decay is at least exp(-scale), so P_16 is at least exp(-16 scale); the host takes these kernels only while
// 16 scale < 13 (P_16 > 2e-6), and products of rows hold P_t / P_j <= 1 for j <= t: nothing overflows and nothing cancels.
//
//   removal_chunk_prepare_kernel   a workgroup per chunk and head: unit keys, removal vectors, the decay's low-rank map, the four
//                                  products, T, and the matrices above into `scratch`
//   removal_chunk_scan_kernel      a workgroup per 16 value columns, head and sequence; a wave holds 16 rows of the state in the
//                                  matrix instructions' result layout, which is also their operand layout, so that the state
//                                  never leaves the registers; the waves exchange their parts of D and O through LDS
#include "common.h"

#define CHUNK 16
#define CHUNK_STRIDE 20  // floats between the rows of a 16 x 16 matrix in LDS (16-byte aligned, rows on different banks)

struct RemovalChunkArgs {
  const void* main;  // [T, ld]
  int ld, r_at, k_at, v_at, a_at, low_at, rank, heads, dim, vdim;
  const float* a_bias;
  const void* w2;
  const float* w0;
  float scale;
  float* scratch;
  float* state;  // [slots, heads, dim, vdim]
  const int* slots;
  const int* cu_q;
  float* out;  // [T, heads * vdim]
};

// A chunk and head in `scratch`, in floats: U' | R' | -B | K (each 16 * dim), P_16 (dim), Dv | Ov | V (each 16 * columns).  U' and R' as
// [dim / 16][16 tokens][16 channels], B and K as [dim][16 tokens], Dv, Ov and V as [columns][16 tokens]: what a wave reads of one
// of them is one contiguous kilobyte, 16 bytes a lane.
__host__ __device__ __forceinline__ int removal_columns(int vdim) { return (vdim + 15) / 16 * 16; }
__host__ __device__ __forceinline__ size_t removal_record(int dim, int vdim) { return (size_t)65 * dim + 48 * removal_columns(vdim); }
// the first record of a sequence: sequences' chunks never overlap, because floor((a + n) / 16) + 1 >= floor(a / 16) + ceil(n / 16)
__device__ __forceinline__ int removal_first_chunk(int first_token, int sequence) { return first_token / CHUNK + sequence; }

__device__ __forceinline__ float removal_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float4_t mfma4(float a, float b, float4_t c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ float4_t four(const float* p) { return *reinterpret_cast<const float4_t*>(p); }

template <typename T>
__global__ void __launch_bounds__(256) removal_chunk_prepare_kernel(const RemovalChunkArgs a) {
  extern __shared__ float4_t lds_pieces[];
  float* lds = reinterpret_cast<float*>(lds_pieces);
  const int h = blockIdx.x, b = blockIdx.z;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  const int t0 = lo + blockIdx.y * CHUNK;
  if (t0 >= hi) return;  // (the whole workgroup)
  const int count = hi - t0 < CHUNK ? hi - t0 : CHUNK;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = lane & 15, g = lane >> 4;  // column and group of four rows in the matrix instructions' layouts
  const int dim = a.dim, rank = a.rank, row = dim + 4;
  const int padded_rank = (rank + 15) / 16 * 16, inner_row = padded_rank + 4;
  // four matrices of 16 rows (U, R, B, K), the decays, the map's inner rows, and 16 x 16 matrices: M1..M4, T, M4 T, T M1
  float* matrix[4] = {lds, lds + CHUNK * row, lds + 2 * CHUNK * row, lds + 3 * CHUNK * row};
  float* decays = lds + 4 * CHUNK * row;
  float* inner = decays + CHUNK * row;
  float* small = inner + CHUNK * inner_row;
  const T* rows = (const T*)a.main + (size_t)t0 * a.ld;

  // a wave takes four tokens and a lane two channels of each (dim <= 128): all of a wave's loads are asked for before the first
  // is used (tokens beyond the portion: zeros, with decays of 1)
  float r[4][2], k[4][2], al[4][2];
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int j = wave + 4 * q;
    const T* mine = rows + (size_t)j * a.ld + (size_t)h * dim;
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int c = lane + 64 * p;
      const bool there = j < count && c < dim;
      r[q][p] = there ? to_f32(mine[a.r_at + c]) : 0.f;
      k[q][p] = there ? to_f32(mine[a.k_at + c]) : 0.f;
      al[q][p] = there ? to_f32(mine[a.a_at + c]) : 0.f;
    }
  }
  const float bias[2] = {lane < dim ? a.a_bias[(size_t)h * dim + lane] : 0.f, lane + 64 < dim ? a.a_bias[(size_t)h * dim + lane + 64] : 0.f};
#pragma unroll 4
  for (int i = tid; i < CHUNK * padded_rank; i += 256) {
    const int j = i / padded_rank, m = i - j * padded_rank;
    inner[j * inner_row + m] = j < count && m < rank ? tanhf(to_f32(rows[(size_t)j * a.ld + a.low_at + m])) : 0.f;
  }
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int j = wave + 4 * q;
    const float inv = 1.f / sqrtf(wave_sum(k[q][0] * k[q][0] + k[q][1] * k[q][1]) + 1e-6f);
#pragma unroll
    for (int p = 0; p < 2; ++p) {
      const int c = lane + 64 * p;
      if (c < dim) {
        const float u = k[q][p] * inv;
        matrix[0][j * row + c] = u;
        matrix[1][j * row + c] = r[q][p];
        matrix[2][j * row + c] = removal_sigmoid(al[q][p] + bias[p]) * u;
        matrix[3][j * row + c] = k[q][p];
      }
    }
  }
  __syncthreads();
  // the decays: 16 channels x 16 tokens at a time, w2 [channel, m] times the inner rows; a lane ends with four neighbouring channels
  // of token n
  for (int tile = wave; tile < dim / 16; tile += 4) {
    const size_t channel = (size_t)h * dim + tile * 16;
    const T* w = (const T*)a.w2 + (channel + n) * rank;
    float4_t z = {0.f, 0.f, 0.f, 0.f};
    if (rank % 16 == 0 && ((uintptr_t)a.w2 & 15) == 0) {  // (then four neighbours of a row are one access)
#pragma unroll 4
      for (int m = 4 * g; m < padded_rank; m += 16) {
        float y[4];
        load4<T>(w, 0, m, rank, true, true, y);
        const float4_t x = four(inner + n * inner_row + m);
#pragma unroll
        for (int e = 0; e < 4; ++e) z = mfma4(y[e], x[e], z);
      }
    } else {
      for (int m = 4 * g; m < padded_rank; m += 16) {
        const float4_t x = four(inner + n * inner_row + m);
#pragma unroll
        for (int e = 0; e < 4; ++e) z = mfma4(m + e < rank ? to_f32(w[m + e]) : 0.f, x[e], z);
      }
    }
    float4_t dec;
#pragma unroll
    for (int i = 0; i < 4; ++i) dec[i] = n < count ? expf(-a.scale * removal_sigmoid(a.w0[channel + 4 * g + i] + z[i])) : 1.f;
    *reinterpret_cast<float4_t*>(decays + n * row + tile * 16 + 4 * g) = dec;
  }
  __syncthreads();
  // the running products and the scaled rows; a lane walks one channel of one of the four matrices
  const int record_at = removal_first_chunk(lo, b) + blockIdx.y;
  float* record = a.scratch + ((size_t)record_at * a.heads + h) * removal_record(dim, a.vdim);
  float* record_b = record + 32 * dim;
  float* record_k = record + 48 * dim;
  float* record_p = record + 64 * dim;
  for (int i = tid; i < 4 * dim; i += 256) {
    const int which = i / dim, c = i - which * dim;
    float* column = matrix[which] + c;
    float p = 1.f;
    float4_t kept[4];
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) {
      const float before = p;
      p *= decays[t * row + c];
      const float v = column[t * row] * (which == 0 ? before : which == 1 ? p : 1.f / p);
      column[t * row] = v;
      kept[t >> 2][t & 3] = which == 2 ? -v : v;
    }
    if (which >= 2) {
      float* to = (which == 2 ? record_b : record_k) + (size_t)c * CHUNK;
#pragma unroll
      for (int q = 0; q < 4; ++q) *reinterpret_cast<float4_t*>(to + 4 * q) = kept[q];
    }
    if (which == 0) record_p[c] = p;
  }
  __syncthreads();
  // M1 = U K^T, M2 = U B^T (below the diagonal), M3 = R K^T, M4 = R B^T (with it): a wave each
  {
    const float* left = matrix[wave < 2 ? 0 : 1] + n * row;
    const float* right = matrix[(wave & 1) ? 2 : 3] + n * row;
    float4_t m = {0.f, 0.f, 0.f, 0.f};
    for (int c = 4 * g; c < dim; c += 16) {
      const float4_t x = four(left + c), y = four(right + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) m = mfma4(x[e], y[e], m);
    }
    float* to = small + wave * CHUNK * CHUNK_STRIDE;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 4 * g + i;
      to[t * CHUNK_STRIDE + n] = n < t || (wave >= 2 && n == t) ? m[i] : 0.f;
    }
  }
  __syncthreads();
  const float* M1 = small;
  const float* M2 = small + CHUNK * CHUNK_STRIDE;
  const float* M3 = small + 2 * CHUNK * CHUNK_STRIDE;
  const float* M4 = small + 3 * CHUNK * CHUNK_STRIDE;
  float* inverse = small + 4 * CHUNK * CHUNK_STRIDE;
  float* M4T = small + 5 * CHUNK * CHUNK_STRIDE;
  float* TM1 = small + 6 * CHUNK * CHUNK_STRIDE;
  if (wave == 0) {  // column n of T, by substitution (the four groups of lanes do the same)
    float x[CHUNK];
#pragma unroll
    for (int t = 0; t < CHUNK; ++t) {
      float v = t == n ? 1.f : 0.f;
#pragma unroll
      for (int q = 0; q < (t + 3) / 4; ++q) {
        const float4_t m = four(M2 + t * CHUNK_STRIDE + 4 * q);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (4 * q + e < t) v -= m[e] * x[4 * q + e];
      }
      x[t] = v;
    }
    if (g == 0) {
#pragma unroll
      for (int t = 0; t < CHUNK; ++t) inverse[t * CHUNK_STRIDE + n] = x[t];
    }
  }
  __syncthreads();
  if (wave < 2) {  // M4 T and T M1
    const float4_t x = four((wave == 0 ? M4 : inverse) + n * CHUNK_STRIDE + 4 * g);
    const float* y = (wave == 0 ? inverse : M1) + 4 * g * CHUNK_STRIDE + n;
    float4_t m = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) m = mfma4(x[e], y[e * CHUNK_STRIDE], m);
    float* to = wave == 0 ? M4T : TM1;
#pragma unroll
    for (int i = 0; i < 4; ++i) to[(4 * g + i) * CHUNK_STRIDE + n] = m[i];
  }
  __syncthreads();
  const float4_t t4 = four(inverse + n * CHUNK_STRIDE + 4 * g), m4t = four(M4T + n * CHUNK_STRIDE + 4 * g);
  for (int tile = wave; tile < dim / 16; tile += 4) {  // U' and R', 16 channels at a time
    float4_t up = {0.f, 0.f, 0.f, 0.f}, rp;
#pragma unroll
    for (int i = 0; i < 4; ++i) rp[i] = matrix[1][(4 * g + i) * row + tile * 16 + n];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float y = matrix[0][(4 * g + e) * row + tile * 16 + n];
      up = mfma4(t4[e], y, up);
      rp = mfma4(-m4t[e], y, rp);
    }
    float* to = record + tile * 256 + n;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      to[(4 * g + i) * 16] = up[i];
      to[16 * dim + (4 * g + i) * 16] = rp[i];
    }
  }
  const float4_t m3 = four(M3 + n * CHUNK_STRIDE + 4 * g), m4 = four(M4 + n * CHUNK_STRIDE + 4 * g), tm1 = four(TM1 + n * CHUNK_STRIDE + 4 * g);
  const int columns = removal_columns(a.vdim);
  float* record_d = record + 65 * dim;
  for (int tile = wave; tile < columns / 16; tile += 4) {  // Dv and Ov, 16 columns of values at a time
    const int column = tile * 16 + n;
    const T* values = rows + a.v_at + (size_t)h * a.vdim + (column < a.vdim ? column : a.vdim - 1);
    float4_t v, dv = {0.f, 0.f, 0.f, 0.f}, ov = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = 4 * g + e < count ? to_f32(values[(size_t)(4 * g + e) * a.ld]) : 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      dv = mfma4(tm1[e], v[e], dv);
      ov = mfma4(m3[e], v[e], ov);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) ov = mfma4(-m4[e], dv[e], ov);
    *reinterpret_cast<float4_t*>(record_d + (size_t)column * CHUNK + 4 * g) = dv;
    *reinterpret_cast<float4_t*>(record_d + (size_t)(columns + column) * CHUNK + 4 * g) = ov;
    *reinterpret_cast<float4_t*>(record_d + (size_t)(2 * columns + column) * CHUNK + 4 * g) = v;
  }
}

// What a wave reads of one chunk, in registers: loaded SCAN_AHEAD chunks before it is worked.
template <int WAVES>
struct RemovalOperands {
  static constexpr int READS = WAVES >= 4 ? 1 : (4 + WAVES - 1) / WAVES;  // read-outs of a chunk that a lane finishes
  float4_t up, rp, nb, k, p, dv, v;
  float ov[READS];
};
#define SCAN_AHEAD 4

// (at most 256 registers a wave: the matrix instructions then keep the state in ordinary registers)
template <int WAVES>
__global__ void __launch_bounds__(64 * WAVES, 2) removal_chunk_scan_kernel(const RemovalChunkArgs a) {
  __shared__ float4_t parts[2][2][WAVES][64];  // [buffer][D, O][wave][lane]
  // (heads lie along the grid's first dimension in both kernels: with a multiple of 8 heads the workgroups that read a record run
  // on the XCD that wrote it and share it in that XCD's L2)
  const int h = blockIdx.x, tile = blockIdx.y, b = blockIdx.z;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  if (hi <= lo) return;  // (the whole workgroup)
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n = lane & 15, g = lane >> 4;
  constexpr int dim = 16 * WAVES;
  constexpr int READS = RemovalOperands<WAVES>::READS;
  const int vdim = a.vdim, columns = removal_columns(vdim);
  const int column = tile * 16 + n;
  const bool live = column < vdim;
  const int chunks = (hi - lo + CHUNK - 1) / CHUNK;
  const size_t stride = (size_t)a.heads * removal_record(dim, vdim);  // between a sequence's records of this head
  // a lane's places in a record, in floats (the record's own address is the same for the whole wave and moves from chunk to chunk)
  const uint32_t rows_at = wave * 256 + n * 16 + 4 * g, decays_at = 64 * dim + wave * 16 + 4 * g, column_at = 65 * dim + column * CHUNK + 4 * g;
  uint32_t reads_at[READS];
#pragma unroll
  for (int q = 0; q < READS; ++q) {
    const int i = (tid + q * 64 * WAVES) & 255;  // a read-out's place in the order in which the parts lie in LDS
    reads_at[q] = 65 * dim + (columns + tile * 16 + ((i >> 2) & 15)) * CHUNK + (i >> 6) * 4 + (i & 3);
  }
  const float* next = a.scratch + ((size_t)removal_first_chunk(lo, b) * a.heads + h) * removal_record(dim, vdim);
  int asked = 0;  // chunks asked for so far
  auto load = [&](RemovalOperands<WAVES>& o) {
    const float* record = next;
    o.up = four(record + rows_at);
    o.rp = four(record + 16 * dim + rows_at);
    o.nb = four(record + 32 * dim + rows_at);
    o.k = four(record + 48 * dim + rows_at);
    o.p = four(record + decays_at);
    o.dv = four(record + column_at);
    o.v = four(record + 32 * columns + column_at);
#pragma unroll
    for (int q = 0; q < READS; ++q) o.ov[q] = record[reads_at[q]];
    ++asked;
    if (asked < chunks) next += stride;  // (beyond the last chunk the last one is asked for again)
  };

  float* S = a.state + (((size_t)a.slots[b] * a.heads + h) * dim + wave * 16 + 4 * g) * vdim + (live ? column : vdim - 1);
  float4_t z;
#pragma unroll
  for (int i = 0; i < 4; ++i) z[i] = S[(size_t)i * vdim];

  const size_t out_row = (size_t)a.heads * vdim;
  float* out = a.out + (size_t)lo * out_row + (size_t)h * vdim + tile * 16;
  int left = hi - lo;  // tokens from the current chunk on

  auto work = [&](int buffer, const RemovalOperands<WAVES>& o) {
    float4_t d = {0.f, 0.f, 0.f, 0.f}, read = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      d = mfma4(o.up[e], z[e], d);
      read = mfma4(o.rp[e], z[e], read);
    }
    parts[buffer][0][wave][lane] = d;
    parts[buffer][1][wave][lane] = read;
#pragma unroll
    for (int e = 0; e < 4; ++e) z = mfma4(o.k[e], o.v[e], z);
    __syncthreads();  // (one a chunk: a buffer is written again behind the next chunk's barrier)
    d = o.dv;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) d += parts[buffer][0][w][lane];
#pragma unroll
    for (int e = 0; e < 4; ++e) z = mfma4(o.nb[e], d[e], z);
    z *= o.p;
    // the chunk's read-outs: 256 of them over the workgroup's lanes
    const float* sums = reinterpret_cast<const float*>(parts[buffer][1]);
#pragma unroll
    for (int q = 0; q < READS; ++q) {
      const int i = tid + q * 64 * WAVES;
      if (i < 256) {
        const int t = (i >> 6) * 4 + (i & 3), e = (i >> 2) & 15;
        float v = o.ov[q];
#pragma unroll
        for (int w = 0; w < WAVES; ++w) v += sums[w * 256 + i];
        if (t < left && tile * 16 + e < vdim) out[t * out_row + e] = v;
      }
    }
    left -= CHUNK;
    out += CHUNK * out_row;
  };

  // Loads are asked for whether or not there is a chunk that far ahead (then the last one's again): the same number of them lies
  // between a chunk's loads and its work on every path, so that waiting for the one does not wait for the others.
  RemovalOperands<WAVES> ops[SCAN_AHEAD];
#pragma unroll
  for (int j = 0; j < SCAN_AHEAD; ++j) load(ops[j]);
  int c = 0;
  for (; c + SCAN_AHEAD <= chunks; c += SCAN_AHEAD) {
#pragma unroll
    for (int j = 0; j < SCAN_AHEAD; ++j) {
      work(j & 1, ops[j]);
      load(ops[j]);
    }
  }
#pragma unroll
  for (int j = 0; j < SCAN_AHEAD - 1; ++j)
    if (c + j < chunks) work(j & 1, ops[j]);  // (the same for the whole workgroup)
  if (live) {
#pragma unroll
    for (int i = 0; i < 4; ++i) S[(size_t)i * vdim] = z[i];
  }
}

static size_t removal_prepare_lds(int dim, int rank) {
  const int padded_rank = (rank + 15) / 16 * 16;
  return (size_t)CHUNK * (5 * (dim + 4) + padded_rank + 4 + 7 * CHUNK_STRIDE) * sizeof(float);
}

// float32 elements of the scratch of a step; 0: these sizes are not for these kernels
extern "C" long long velox_removal_chunk_scratch_elems(int tokens, int num_seqs, int heads, int dim, int vdim, int rank) {
  if (dim % 16 != 0 || dim < 16 || dim > 128 || vdim < 1 || rank < 1 || removal_prepare_lds(dim, rank) > 64 * 1024) return 0;
  return ((long long)tokens / CHUNK + num_seqs + 1) * heads * (long long)removal_record(dim, vdim);
}

template <typename T>
static void removal_chunk_launch(const RemovalChunkArgs& a, int num_seqs, int max_q_len, hipStream_t stream) {
  const int chunks = (max_q_len + CHUNK - 1) / CHUNK;
  removal_chunk_prepare_kernel<T><<<dim3(a.heads, chunks, num_seqs), 256, removal_prepare_lds(a.dim, a.rank), stream>>>(a);
  const dim3 grid(a.heads, removal_columns(a.vdim) / 16, num_seqs);
  switch (a.dim / 16) {
    case 1: removal_chunk_scan_kernel<1><<<grid, 64, 0, stream>>>(a); break;
    case 2: removal_chunk_scan_kernel<2><<<grid, 128, 0, stream>>>(a); break;
    case 3: removal_chunk_scan_kernel<3><<<grid, 192, 0, stream>>>(a); break;
    case 4: removal_chunk_scan_kernel<4><<<grid, 256, 0, stream>>>(a); break;
    case 5: removal_chunk_scan_kernel<5><<<grid, 320, 0, stream>>>(a); break;
    case 6: removal_chunk_scan_kernel<6><<<grid, 384, 0, stream>>>(a); break;
    case 7: removal_chunk_scan_kernel<7><<<grid, 448, 0, stream>>>(a); break;
    default: removal_chunk_scan_kernel<8><<<grid, 512, 0, stream>>>(a); break;
  }
}

extern "C" int velox_removal_chunk_scan(const void* main, int dtype, int ld, int r_at, int k_at, int v_at, int a_at, int low_at, int rank, int heads, int dim,
                                        int vdim, const float* a_bias, const void* w2, const float* w0, float scale, float* scratch, float* state,
                                        const int* slots, const int* cu_q, float* out, int num_seqs, int max_q_len, hipStream_t stream) {
  if (num_seqs <= 0 || max_q_len <= 0) return 0;
  if (velox_removal_chunk_scratch_elems(max_q_len, num_seqs, heads, dim, vdim, rank) == 0 || heads < 1 || heads > 65535 || num_seqs > 65535 ||
      max_q_len > 65535 * CHUNK || !scratch || !(scale * CHUNK < 13.f))
    return (int)hipErrorInvalidValue;
  RemovalChunkArgs a{main, ld, r_at, k_at, v_at, a_at, low_at, rank, heads, dim, vdim, a_bias, w2, w0, scale, scratch, state, slots, cu_q, out};
  if (dtype == VELOX_BF16) removal_chunk_launch<bf16_t>(a, num_seqs, max_q_len, stream);
  else removal_chunk_launch<float>(a, num_seqs, max_q_len, stream);
  VELOX_RETURN_LAUNCH_STATUS();
}
