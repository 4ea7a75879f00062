// gated_scan: a recurrence on every channel by itself, S_t = (1 - z_t) S_(t-1) + z_t c_t, whose gates read only the current token.
//   A row of `proj` holds z, u and g, `width` channels each:  z = sigmoid(proj_z + bias_z);  u = proj_u + bias_u;
//   c = u + shift (u >= 0) or sigmoid(u) (u < 0);  out[t] = S_t * silu(g).  The state is float32 [slots, width].
// Everything between a load and a store is float32.
//
// Steps whose portions fit one piece of GATED_PIECE tokens (decoding, short portions): one lane per channel (or two
// neighbouring channels) walks the portion from the slot's state.  Longer portions are cut into pieces that are worked at
// the same time, in two passes over the rows:
//   gated_pieces_kernel: per piece and channel A = product of (1 - z) and B = the state the piece reaches from zero, into `scratch`
//     [sequence][1 + pieces][2][width]; the first entry is (0, the slot's state), which only this pass reads;
//   gated_scan_kernel: every piece folds the entries before it into the state it starts from, walks its tokens and writes
//     the outputs; a sequence's last piece writes the slot's state.
#include "common.h"

#define GATED_PIECE 64

struct GatedArgs {
  const void* proj;
  int width;
  const float* bias_z;
  const float* bias_u;
  float shift;
  float* state;
  const int* slots;
  const int* cu_q;
  void* out;
  float* scratch;  // nullptr: portions of one piece
  int entries;     // 1 + the pieces of the longest portion
};

// V neighbouring channels of a row, widened
template <typename T, int V>
__device__ __forceinline__ void load_channels(const T* __restrict__ p, float (&v)[V]) {
  if constexpr (V == 2 && sizeof(T) == 2) {
    const uint32_t raw = *reinterpret_cast<const uint32_t*>(p);
    v[0] = __uint_as_float(raw << 16);
    v[1] = __uint_as_float(raw & 0xffff0000u);
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = to_f32(p[i]);
  }
}
template <typename T, int V>
__device__ __forceinline__ void store_channels(T* __restrict__ p, const float (&v)[V]) {
  if constexpr (V == 2 && sizeof(T) == 2) {
    *reinterpret_cast<uint32_t*>(p) = (uint32_t)(uint16_t)bf16_bits(v[0]) | ((uint32_t)(uint16_t)bf16_bits(v[1]) << 16);
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) p[i] = from_f32<T>(v[i]);
  }
}

__device__ __forceinline__ float gated_sigmoid(float x) { return 1.f / (1.f + expf(-x)); }

// keep = 1 - z and add = z * candidate of one token and channel; 1 - sigmoid(x) is taken as sigmoid(-x), which loses nothing near 0
__device__ __forceinline__ void gated_token(float xz, float xu, float shift, float& keep, float& add) {
  keep = gated_sigmoid(-xz);
  add = gated_sigmoid(xz) * (xu >= 0.f ? xu + shift : gated_sigmoid(xu));
}

#define GATED_AHEAD 4  // tokens whose loads are in flight together

template <typename T, int V>
__global__ void __launch_bounds__(128) gated_pieces_kernel(const GatedArgs a) {
  const int c = (blockIdx.x * 128 + threadIdx.x) * V;
  const int b = blockIdx.z, piece = blockIdx.y, W = a.width;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  const int first = lo + piece * GATED_PIECE;
  if (c >= W || first >= hi) return;
  float* entry = a.scratch + (size_t)b * a.entries * 2 * W + c;
  if (piece == 0) {
#pragma unroll
    for (int i = 0; i < V; ++i) {
      entry[i] = 0.f;
      entry[W + i] = a.state[(size_t)a.slots[b] * W + c + i];
    }
  }
  if (first + GATED_PIECE >= hi) return;  // (a last piece: nobody folds it)
  float bz[V], bu[V], A[V], B[V];
#pragma unroll
  for (int i = 0; i < V; ++i) { bz[i] = a.bias_z[c + i]; bu[i] = a.bias_u[c + i]; A[i] = 1.f; B[i] = 0.f; }
  const T* row = (const T*)a.proj + (size_t)first * 3 * W + c;
  for (int t = 0; t < GATED_PIECE; t += GATED_AHEAD) {
    float z[GATED_AHEAD][V], u[GATED_AHEAD][V];
#pragma unroll
    for (int j = 0; j < GATED_AHEAD; ++j) {
      load_channels<T, V>(row + (size_t)(t + j) * 3 * W, z[j]);
      load_channels<T, V>(row + (size_t)(t + j) * 3 * W + W, u[j]);
    }
#pragma unroll
    for (int j = 0; j < GATED_AHEAD; ++j)
#pragma unroll
      for (int i = 0; i < V; ++i) {
        float keep, add;
        gated_token(z[j][i] + bz[i], u[j][i] + bu[i], a.shift, keep, add);
        A[i] *= keep;
        B[i] = keep * B[i] + add;
      }
  }
  entry += (size_t)(piece + 1) * 2 * W;
#pragma unroll
  for (int i = 0; i < V; ++i) { entry[i] = A[i]; entry[W + i] = B[i]; }
}

template <typename T, int V>
__global__ void __launch_bounds__(128) gated_scan_kernel(const GatedArgs a) {
  const int c = (blockIdx.x * 128 + threadIdx.x) * V;
  const int b = blockIdx.z, piece = blockIdx.y, W = a.width;
  const int lo = a.cu_q[b], hi = a.cu_q[b + 1];
  const int first = lo + piece * GATED_PIECE;
  if (c >= W || first >= hi) return;
  const int last = first + GATED_PIECE < hi ? first + GATED_PIECE : hi;
  float* my_state = a.state + (size_t)a.slots[b] * W + c;
  float bz[V], bu[V], s[V];
#pragma unroll
  for (int i = 0; i < V; ++i) { bz[i] = a.bias_z[c + i]; bu[i] = a.bias_u[c + i]; s[i] = 0.f; }
  if (a.scratch) {
    const float* entry = a.scratch + (size_t)b * a.entries * 2 * W + c;
    for (int p = 0; p <= piece; ++p, entry += 2 * (size_t)W) {
#pragma unroll
      for (int i = 0; i < V; ++i) s[i] = entry[i] * s[i] + entry[W + i];
    }
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) s[i] = my_state[i];
  }
  const T* row = (const T*)a.proj + c;
  T* out = (T*)a.out + c;
  for (int t = first; t < last; t += GATED_AHEAD) {
    float z[GATED_AHEAD][V], u[GATED_AHEAD][V], g[GATED_AHEAD][V];
#pragma unroll
    for (int j = 0; j < GATED_AHEAD; ++j) {
      const size_t at = (size_t)(t + j < last ? t + j : last - 1) * 3 * W;  // (a place beyond the portion follows its last token and is not worked)
      load_channels<T, V>(row + at, z[j]);
      load_channels<T, V>(row + at + W, u[j]);
      load_channels<T, V>(row + at + 2 * W, g[j]);
    }
#pragma unroll
    for (int j = 0; j < GATED_AHEAD; ++j) {
      if (t + j < last) {
        float o[V];
#pragma unroll
        for (int i = 0; i < V; ++i) {
          float keep, add;
          gated_token(z[j][i] + bz[i], u[j][i] + bu[i], a.shift, keep, add);
          s[i] = keep * s[i] + add;
          o[i] = s[i] * (g[j][i] * gated_sigmoid(g[j][i]));
        }
        store_channels<T, V>(out + (size_t)(t + j) * W, o);
      }
    }
  }
  if (last == hi) {
#pragma unroll
    for (int i = 0; i < V; ++i) my_state[i] = s[i];
  }
}

// float32 elements of the scratch that a step with portions of at most max_q_len tokens needs (0: none)
extern "C" long long velox_gated_scan_scratch_elems(int num_seqs, int max_q_len, int width) {
  const long long pieces = (max_q_len + GATED_PIECE - 1) / GATED_PIECE;
  return pieces <= 1 ? 0 : (long long)num_seqs * (1 + pieces) * 2 * width;
}

template <typename T, int V>
static void gated_scan_launch(const GatedArgs& a, int pieces, int num_seqs, hipStream_t stream) {
  const dim3 grid((a.width + 128 * V - 1) / (128 * V), pieces, num_seqs);
  if (a.scratch) gated_pieces_kernel<T, V><<<grid, 128, 0, stream>>>(a);
  gated_scan_kernel<T, V><<<grid, 128, 0, stream>>>(a);
}

extern "C" int velox_gated_scan(const void* proj, int dtype, int width, const float* bias_z, const float* bias_u, float shift, float* state, const int* slots,
                                const int* cu_q, void* out, float* scratch, int num_seqs, int max_q_len, hipStream_t stream) {
  if (num_seqs <= 0 || max_q_len <= 0) return 0;
  const int pieces = (max_q_len + GATED_PIECE - 1) / GATED_PIECE;
  if (width < 1 || num_seqs > 65535 || pieces > 65535 || (pieces > 1 && !scratch)) return (int)hipErrorInvalidValue;
  GatedArgs a{proj, width, bias_z, bias_u, shift, state, slots, cu_q, out, pieces > 1 ? scratch : nullptr, 1 + pieces};
  // two neighbouring channels a lane where rows allow it and the step is long enough to be bound by its bytes
  const bool pairs = pieces > 1 && width % 2 == 0 && (((uintptr_t)proj | (uintptr_t)out) & 3) == 0;
  if (dtype == VELOX_BF16) {
    if (pairs) gated_scan_launch<bf16_t, 2>(a, pieces, num_seqs, stream);
    else gated_scan_launch<bf16_t, 1>(a, pieces, num_seqs, stream);
  } else {
    gated_scan_launch<float, 1>(a, pieces, num_seqs, stream);
  }
  VELOX_RETURN_LAUNCH_STATUS();
}
