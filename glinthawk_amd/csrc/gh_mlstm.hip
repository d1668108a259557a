// Matrix-memory LSTM (the mLSTM of xLSTM: Beck et al., "xLSTM: Extended Long Short-Term Memory"): exponential input gate and sigmoid
// forget gate in log space with a running maximum m (starting at 0), a matrix S and a vector n per head.
//
//   m' = max(f + m, i);  S' = e^(f + m - m') S + e^(i - m') k v^T;  n' likewise with k;  o = S'^T q / (max(|n' . q|, e^(-m')) + 1e-6)
//
// gates   i = cap tanh((. + b) / cap), f = logsigmoid(cap tanh((. + b) / cap))
// state   fp32, per context and head: S (dim x vdim_padded), then n (heads x dim), then m (heads); zero at position 0, which the kernels
//         take from the position (a slot that is used again needs no clearing)
// walk    work-group = 64 columns of v of one (context, head); it keeps its (dim x 64) part of S in registers over all the tokens of the
//         call (one for decode) and streams it in and out of memory once.  n and m are needed by every column slice: each slice carries
//         its own copy and the finishing kernel writes them back, so no slice reads what another one has already replaced.
// finish  one work-group per token: each head's output divided by its root mean square, times a weight, times sigmoid(g)
#include "gh_product.h"

#include <algorithm>
#include <type_traits>

namespace gh {
namespace {

constexpr uint32_t SLICE = 64;          // columns of v per work-group
constexpr uint32_t CHUNKED_TOKENS = 24; // from this many tokens per context on, bf16 runs in chunks on the matrix cores

struct MlstmShape
{
  uint32_t heads, dim, vdim, vpad;
  float cap, eps, q_scale;
  // elements of the state of one context
  __host__ __device__ uint64_t n_off() const { return (uint64_t)heads * dim * vpad; }
  __host__ __device__ uint64_t m_off() const { return n_off() + (uint64_t)heads * dim; }
  __host__ __device__ uint64_t elements() const { return m_off() + heads; }
};

__device__ __forceinline__ float soft_cap( float z, float cap ) { return cap * tanhf( z / cap ); }
// log(sigmoid(z)), stable for either sign
__device__ __forceinline__ float log_sigmoid( float z ) { return fminf( z, 0.0f ) - log1pf( expf( -fabsf( z ) ) ); }

// columns of the products: [q | k | v | g] in one, [i | f] in the other
struct MlstmCols
{
  uint32_t q, k, v, g, i, f;
};

// `gates`: (rows, 2 heads) fp32, the log input gates of a token's heads, then its log forget gates (mlstm_gates_kernel)
template<typename E, typename View>
struct MlstmIn
{
  View main;
  const float* gates;
  MlstmCols col;
};

template<typename E>
__global__ __launch_bounds__( 256 ) void mlstm_gates_kernel( float* __restrict__ out,
                                                             ProductView<float> y,
                                                             MlstmCols col,
                                                             const E* __restrict__ bias_i,
                                                             const E* __restrict__ bias_f,
                                                             uint32_t heads,
                                                             uint64_t rows,
                                                             float cap )
{
  const uint64_t total = rows * 2 * heads, stride = (uint64_t)gridDim.x * blockDim.x;
  for ( uint64_t i = (uint64_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += stride ) {
    const uint64_t row = i / ( 2 * heads );
    const uint32_t g = (uint32_t)( i % ( 2 * heads ) ), h = g < heads ? g : g - heads;
    const E* bias = g < heads ? bias_i : bias_f;
    const float z = soft_cap( y.at( row, ( g < heads ? col.i : col.f ) + h ) + ( bias != nullptr ? to_f32( bias[h] ) : 0.0f ), cap );
    out[i] = g < heads ? z : log_sigmoid( z );
  }
}

struct MlstmState
{
  void* const* rows;         // state region of each context; NULL: no context
  uint64_t offset;           // bytes from there to this layer's state
  const uint32_t* start_pos; // position of the first token of the call
  uint32_t n_tokens;
};

// RPT: rows of S per thread kept in registers (0: S stays in memory, any dim)
template<typename E, typename View, int RPT>
__global__ __launch_bounds__( 256 ) void mlstm_walk_kernel( float* __restrict__ o_out, float* __restrict__ nm_out, MlstmIn<E, View> in, MlstmState st, MlstmShape s )
{
  extern __shared__ float lds[];
  const uint32_t dim4 = ( s.dim + 3 ) / 4 * 4; // v_s and red are read as float4
  float* q_s = lds;               // dim
  float* k_s = q_s + dim4;        // dim
  float* n_s = k_s + dim4;        // dim
  float* v_s = n_s + s.dim;       // SLICE
  float* nq_s = v_s + SLICE;      // 16
  float* red = nq_s + 16;         // 16 x SLICE
  const uint32_t slice = blockIdx.x, h = blockIdx.y, ctx = blockIdx.z;
  uint8_t* base = static_cast<uint8_t*>( st.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  float* S = reinterpret_cast<float*>( base + st.offset );
  const float* n_in = S + s.n_off() + (uint64_t)h * s.dim;
  const float* m_in = S + s.m_off() + h;
  S += (uint64_t)h * s.dim * s.vpad;
  const bool fresh = st.start_pos[ctx] == 0;
  const uint32_t t = threadIdx.x;
  const uint32_t cl = t & 15, rg = t >> 4;
  const uint32_t c0 = slice * SLICE + cl * 4;
  const bool col_live = c0 < s.vpad;
  constexpr int R = RPT > 0 ? RPT : 1;
  float4 reg[R];
  if constexpr ( RPT > 0 ) {
#pragma unroll
    for ( int r = 0; r < RPT; r++ ) {
      const uint32_t row = rg + 16 * r;
      reg[r] = make_float4( 0.0f, 0.0f, 0.0f, 0.0f );
      if ( !fresh && row < s.dim && col_live ) {
        reg[r] = *reinterpret_cast<const float4*>( S + (uint64_t)row * s.vpad + c0 );
      }
    }
  } else if ( fresh && col_live ) {
    for ( uint32_t row = rg; row < s.dim; row += 16 ) {
      *reinterpret_cast<float4*>( S + (uint64_t)row * s.vpad + c0 ) = make_float4( 0.0f, 0.0f, 0.0f, 0.0f );
    }
  }
  for ( uint32_t d = t; d < s.dim; d += 256 ) {
    n_s[d] = fresh ? 0.0f : n_in[d];
  }
  float m = fresh ? 0.0f : *m_in;

  for ( uint32_t tok = 0; tok < st.n_tokens; tok++ ) {
    const uint64_t row_in = (uint64_t)ctx * st.n_tokens + tok;
    __syncthreads(); // the previous token's readers are done (and n_s is written)
    for ( uint32_t d = t; d < s.dim; d += 256 ) {
      q_s[d] = in.main.at( row_in, in.col.q + h * s.dim + d ) * s.q_scale;
      k_s[d] = in.main.at( row_in, in.col.k + h * s.dim + d );
    }
    if ( t < SLICE ) {
      const uint32_t c = slice * SLICE + t;
      v_s[t] = c < s.vdim ? in.main.at( row_in, in.col.v + h * s.vdim + c ) : 0.0f;
    }
    const float gi = in.gates[row_in * 2 * s.heads + h], gf = in.gates[( row_in * 2 + 1 ) * s.heads + h];
    const float m_new = fmaxf( gf + m, gi );
    const float decay = expf( gf + m - m_new ), inp = expf( gi - m_new );
    m = m_new;
    __syncthreads();
    const float4 v4 = *reinterpret_cast<const float4*>( v_s + cl * 4 );
    float4 acc = make_float4( 0.0f, 0.0f, 0.0f, 0.0f );
    auto row_step = [&]( float4& x, uint32_t row ) {
      const float kk = inp * k_s[row], qq = q_s[row];
      x.x = decay * x.x + kk * v4.x;
      x.y = decay * x.y + kk * v4.y;
      x.z = decay * x.z + kk * v4.z;
      x.w = decay * x.w + kk * v4.w;
      acc.x += qq * x.x;
      acc.y += qq * x.y;
      acc.z += qq * x.z;
      acc.w += qq * x.w;
    };
    if constexpr ( RPT > 0 ) {
#pragma unroll
      for ( int r = 0; r < RPT; r++ ) {
        const uint32_t row = rg + 16 * r;
        if ( row < s.dim ) {
          row_step( reg[r], row );
        }
      }
    } else if ( col_live ) {
      for ( uint32_t row = rg; row < s.dim; row += 16 ) {
        float4* p = reinterpret_cast<float4*>( S + (uint64_t)row * s.vpad + c0 );
        float4 x = *p;
        row_step( x, row );
        *p = x;
      }
    }
    // n: one owner per element; its product with q by the sixteen row groups
    float nq = 0.0f;
    for ( uint32_t row = rg + 16 * cl; row < s.dim; row += 256 ) {
      const float x = decay * n_s[row] + inp * k_s[row];
      n_s[row] = x;
      nq += x * q_s[row];
    }
    nq = row16_sum( nq );
    if ( cl == 0 ) {
      nq_s[rg] = nq;
    }
    *reinterpret_cast<float4*>( red + rg * SLICE + cl * 4 ) = acc;
    __syncthreads();
    if ( t < SLICE && slice * SLICE + t < s.vdim ) {
      float num = 0.0f, den = 0.0f;
#pragma unroll
      for ( int r = 0; r < 16; r++ ) {
        num += red[r * SLICE + t];
        den += nq_s[r];
      }
      o_out[row_in * s.heads * s.vdim + h * s.vdim + slice * SLICE + t] = num / ( fmaxf( fabsf( den ), expf( -m ) ) + 1e-6f );
    }
  }
  if constexpr ( RPT > 0 ) {
#pragma unroll
    for ( int r = 0; r < RPT; r++ ) {
      const uint32_t row = rg + 16 * r;
      if ( row < s.dim && col_live ) {
        *reinterpret_cast<float4*>( S + (uint64_t)row * s.vpad + c0 ) = reg[r];
      }
    }
  }
  if ( slice == 0 ) {
    float* dst = nm_out + ( (uint64_t)ctx * s.heads + h ) * ( s.dim + 1 );
    for ( uint32_t row = t; row < s.dim; row += 256 ) { // (the owners wrote before the last barrier)
      dst[row] = n_s[row];
    }
    if ( t == 0 ) {
      dst[s.dim] = m;
    }
  }
}

// ---- many tokens: chunks of 64 on the matrix cores (bf16 products) -------------------------------------------------------------
//
// With b_t the sum of the log forget gates of the chunk up to token t, c_s = i_s - b_s and M_t = max(m0, c_1 .. c_t) (m0: the running
// maximum in front of the chunk), the recurrence unrolls to m_t = b_t + M_t and
//
//   S_t = e^(m0 - M_t) S_0 + sum_(s <= t) e^(c_s - M_t) k_s v_s^T                      (n_t likewise)
//   o_t = (e^(m0 - M_t) S_0^T q_t + sum_(s <= t) e^(c_s - M_t) (k_s . q_t) v_s) / (max(|n_t . q_t|, e^(-m_t)) + 1e-6)
//
// work-group  2 waves on one (context, head, 64 columns of v) walk the chunks; a wave owns 32 columns, its part of S (dim x 32, fp32) stays in
//             accumulator registers from the first chunk to the last.  Two work-groups per CU cover each other's loads.
// exactness   q, k, v are bf16 already.  What enters the state (the weighted values) meets k as three bf16 terms, 24 bits: the state's sums are
//             those of fp32 operands at the rate of bf16 matrix instructions.  What is read out of it for the output (S, the weights of
//             the keys) meets q and v as two terms, 16 bits.  n is carried in fp32, each wave half of it.
// loads       k of a chunk is requested at its head, q and v of the next one as soon as both waves have read this one's.
// operands    an accumulator tile of v_mfma_f32_32x32x16_bf16 (lane = column, registers = rows 8 (v / 4) + 4 (lane / 32) + v % 4) is, as it
//             lies, an operand of the next product over those rows when the other operand takes its sixteen k in the same order:
//               scores^T = K Q^T        lane = query, registers = keys   -> left operand of   P V     (V out of LDS transposed)
//               S                       lane = column of v, registers = dim -> right operand of Q S   (Q out of LDS in pieces of 4)
//             S += K^T (w V): both operands out of LDS with transposing reads (ds_read_b64_tr_b16).
// LDS         64 rows each of q, k (16-byte chunks XORed with bits of the row, so that row reads and transposing reads both spread over
//             the banks) and of v, straight from memory (buffer_load ... lds; rows past the sequence and padding read as zero).
constexpr int CHUNK = 64;
typedef __attribute__( ( address_space( 3 ) ) ) void* lds_ptr;
typedef __attribute__( ( address_space( 3 ) ) ) char lds_char;
typedef short v4s __attribute__( ( ext_vector_type( 4 ) ) );
typedef __attribute__( ( address_space( 3 ) ) ) v4s* lds_v4s;
typedef Mfma<__bf16>::x8 bf16x8;

// slot of 16-byte chunk `chunk` of row `row` in a tile of DT * 4 chunks a row
template<int DT>
__device__ __forceinline__ uint32_t swizzle( uint32_t row, uint32_t chunk )
{
  return DT == 2 ? chunk ^ ( ( ( ( row >> 1 ) & 1 ) << 2 ) | ( ( row >> 2 ) & 3 ) ) : chunk ^ ( ( ( row & 3 ) << 2 ) | ( ( row >> 2 ) & 3 ) );
}
__device__ __forceinline__ uint32_t swizzle_v( uint32_t row, uint32_t chunk ) { return chunk ^ ( 4 * ( ( row >> 1 ) & 1 ) ); }

// Eight fp32 values as N bf16 terms each, 8 bits of mantissa a term; taken two at a time, as the conversion instruction does.
typedef float f32x2 __attribute__( ( ext_vector_type( 2 ) ) );
typedef __bf16 bf16x2 __attribute__( ( ext_vector_type( 2 ) ) );
template<int N>
struct Split
{
  union
  {
    bf16x2 pair[4];
    bf16x8 x;
  } t[N];
  __device__ __forceinline__ void set( int k, float x0, float x1 ) // elements 2 k, 2 k + 1
  {
#pragma unroll
    for ( int n = 0; n < N; n++ ) {
      const bf16x2 b = __builtin_convertvector( ( f32x2 { x0, x1 } ), bf16x2 );
      t[n].pair[k] = b;
      x0 -= (float)b[0];
      x1 -= (float)b[1];
    }
  }
};
template<int N>
__device__ __forceinline__ mfma_f32x16 mma( const bf16x8 a, const Split<N>& b, mfma_f32x16 c )
{
#pragma unroll
  for ( int n = N - 1; n >= 0; n-- ) {
    c = Mfma<__bf16>::k16( a, b.t[n].x, c );
  }
  return c;
}
template<int N>
__device__ __forceinline__ mfma_f32x16 mma( const Split<N>& a, const bf16x8 b, mfma_f32x16 c )
{
#pragma unroll
  for ( int n = N - 1; n >= 0; n-- ) {
    c = Mfma<__bf16>::k16( a.t[n].x, b, c );
  }
  return c;
}
__device__ __forceinline__ double shfl_up_f64( double v, int by )
{
  const uint64_t bits = __builtin_bit_cast( uint64_t, v );
  const uint32_t lo = __shfl_up( (uint32_t)bits, by ), hi = __shfl_up( (uint32_t)( bits >> 32 ), by );
  return __builtin_bit_cast( double, ( (uint64_t)hi << 32 ) | lo );
}
__device__ __forceinline__ double last_lane_f64( double v )
{
  const uint64_t bits = __builtin_bit_cast( uint64_t, v );
  const uint32_t lo = __builtin_amdgcn_readlane( (uint32_t)bits, 63 ), hi = __builtin_amdgcn_readlane( (uint32_t)( bits >> 32 ), 63 );
  return __builtin_bit_cast( double, ( (uint64_t)hi << 32 ) | lo );
}

// DT: 32-row tiles of S, dim <= 32 DT.  dim % 8 == 0, vdim % 8 == 0, 16-byte aligned product rows.
template<int DT>
__global__ __launch_bounds__( 128, 1 ) void mlstm_chunk_kernel( float* __restrict__ o_out, float* __restrict__ nm_out, MlstmIn<__bf16, ProductView<__bf16>> in, MlstmState st,
                                                                MlstmShape s, uint32_t slices, uint32_t n_pairs )
{
  constexpr uint32_t RB = DT * 64; // bytes of a q or k row in LDS
  __shared__ uint4 s_k[CHUNK * RB / 16], s_q[CHUNK * RB / 16];
  __shared__ uint4 s_v[CHUNK * 8];
  __shared__ float s_n[32 * DT];                                      // a wave reads and writes its half only
  __shared__ __attribute__( ( aligned( 16 ) ) ) float s_nq[2][CHUNK]; // n . q over each wave's half; everything below: each wave its own copy
  __shared__ __attribute__( ( aligned( 16 ) ) ) float s_c[2][CHUNK]; // c_s - M of the chunk's last token, s_w: e to the power of it
  __shared__ __attribute__( ( aligned( 16 ) ) ) float s_w[2][CHUNK];
  __shared__ __attribute__( ( aligned( 16 ) ) ) float s_a[2][CHUNK];   // factor of the state in front of the chunk, per token
  __shared__ __attribute__( ( aligned( 16 ) ) ) float s_inv[2][CHUNK]; // one over the denominator

  // the slices of a (context, head) read the same q and k: all on one XCD, next to each other in time
  const uint32_t pair = ( blockIdx.x >> 3 ) / slices * 8 + ( blockIdx.x & 7 ), slice = ( blockIdx.x >> 3 ) % slices;
  if ( pair >= n_pairs ) {
    return;
  }
  const uint32_t h = pair % s.heads, ctx = pair / s.heads;
  uint8_t* base = static_cast<uint8_t*>( st.rows[ctx] );
  if ( base == nullptr ) {
    return;
  }
  float* S_mem = reinterpret_cast<float*>( base + st.offset );
  const float* n_in = S_mem + s.n_off() + (uint64_t)h * s.dim;
  const float m_mem = S_mem[s.m_off() + h];
  S_mem += (uint64_t)h * s.dim * s.vpad;
  const bool fresh = st.start_pos[ctx] == 0;
  const uint32_t wave = __builtin_amdgcn_readfirstlane( threadIdx.x >> 6 );
  const uint32_t lane = threadIdx.x & 63, r = lane & 31, g2 = lane >> 5;
  const uint32_t col = slice * 64 + wave * 32 + r; // this lane's column of v

  constexpr uint32_t PAST_THE_END = 0x80000000u; // an offset beyond any descriptor: reads zero, stores nothing
  const __amdgpu_buffer_rsrc_t S_rsrc = __builtin_amdgcn_make_buffer_rsrc( S_mem, 0, (int)( s.dim * s.vpad * 4 ), 0x00020000 );
  const uint32_t S_off = col < s.vpad ? ( 4 * g2 * s.vpad + col ) * 4 : PAST_THE_END;
  mfma_f32x16 S[DT];
#pragma unroll
  for ( int dt = 0; dt < DT; dt++ ) {
#pragma unroll
    for ( int v = 0; v < 16; v++ ) {
      S[dt][v] = __builtin_bit_cast( float, __builtin_amdgcn_raw_buffer_load_b32( S_rsrc, fresh ? PAST_THE_END : S_off, ( 32 * dt + 8 * ( v / 4 ) + v % 4 ) * s.vpad * 4, 0 ) );
    }
  }
  for ( uint32_t d = threadIdx.x; d < 32 * DT; d += 128 ) {
    s_n[d] = !fresh && d < s.dim ? n_in[d] : 0.0f;
  }
  double m0 = fresh ? 0.0 : (double)m_mem;
  const uint64_t row_first = (uint64_t)ctx * st.n_tokens;
  const uint32_t ld_bytes = (uint32_t)( in.main.stride * 2 );

  // LDS byte addresses: a part that depends on the lane, a constant, and a constant XORed with a lane value (the swizzle acts on the
  // sixteen slots of 256 bytes, or eight of 128).  Computed where they are used: kept in registers over the loop there are too many of them.
  constexpr uint32_t PERIOD = DT == 2 ? 128 : 256;
  auto slot_at = [&]( uint32_t constant, uint32_t lane_xor ) __attribute__( ( always_inline ) ) {
    return constant / PERIOD * PERIOD + ( ( constant % PERIOD ) ^ lane_xor );
  };
  auto opaque = []( uint32_t v ) __attribute__( ( always_inline ) ) {
    asm volatile( "" : "+v"( v ) );
    return v;
  };
  const uint32_t row_swz = swizzle<DT>( r, 0 ) * 16; // of rows r and r + 32

  // rows [0, rows) x `chunks` 16-byte chunks of the product at `p`, LDS rows of 64 DT (or, for v, 128) bytes; the rest reads as zero
  auto fetch = [&]( uint4* tile, const __bf16* p, uint32_t rows, uint32_t chunks, auto slot_of, auto row_bytes_tag ) {
    constexpr uint32_t BYTES = decltype( row_bytes_tag )::value;
    const __amdgpu_buffer_rsrc_t rsrc
      = __builtin_amdgcn_make_buffer_rsrc( const_cast<__bf16*>( p ), 0, (int)( rows > 0 ? ( rows - 1 ) * ld_bytes + chunks * 16 : 0 ), 0x00020000 );
    constexpr uint32_t ROWS = 1024 / BYTES; // rows of one instruction of one wave
    const uint32_t ln = opaque( lane );
#pragma unroll
    for ( uint32_t i = 0; i < CHUNK / ( 2 * ROWS ); i++ ) {
      const uint32_t row0 = ( 2 * i + wave ) * ROWS;
      const uint32_t row = row0 + ln / ( BYTES / 16 );
      const uint32_t chunk = slot_of( row, ln % ( BYTES / 16 ) ); // the swizzle is its own inverse
      const uint32_t off = chunk < chunks ? row * ld_bytes + chunk * 16 : PAST_THE_END;
      __builtin_amdgcn_raw_ptr_buffer_load_lds( rsrc, (lds_ptr)( tile + row0 * ( BYTES / 16 ) ), 16, off, 0, 0, 0 );
    }
  };

  auto swizzle_row = []( uint32_t row, uint32_t c ) { return swizzle<DT>( row, c ); };
  auto fetch_qv = [&]( uint32_t t0 ) {
    const uint32_t rows = min( (uint32_t)CHUNK, st.n_tokens - t0 );
    const __bf16* first = in.main.data + ( row_first + t0 ) * in.main.stride;
    fetch( s_q, first + in.col.q + h * s.dim, rows, s.dim / 8, swizzle_row, std::integral_constant<uint32_t, RB> {} );
    fetch( s_v, first + in.col.v + h * s.vdim + slice * 64, rows, min( 8u, ( s.vdim - slice * 64 ) / 8 ), swizzle_v, std::integral_constant<uint32_t, 128> {} );
  };

  // transposing reads: lane j = 4 e + q of a 16-lane group points at row e (0..3) of its half-wave's four, dims 16 grp + 4 q .. + 3
  const uint32_t tr_e = ( lane & 15 ) >> 2, tr_q = lane & 3, tr_grp = ( lane >> 4 ) & 1;
  const uint32_t trk_row = ( 4 * g2 + tr_e ) * RB + ( tr_q & 1 ) * 8, trk_swz = ( swizzle<DT>( 4 * g2 + tr_e, 2 * tr_grp + ( tr_q >> 1 ) ) ) * 16;
  auto tr_k = [&]( int kk, int dt, uint32_t row, uint32_t swz ) __attribute__( ( always_inline ) ) {
    union
    {
      v4s half[2];
      bf16x8 x;
    } u;
#pragma unroll
    for ( int hf = 0; hf < 2; hf++ ) { // rows 8 further on: bit 1 of the swizzle's low part
      u.half[hf] = __builtin_amdgcn_ds_read_tr16_b64_v4i16( (lds_v4s)( (lds_char*)s_k + row + ( 16 * kk + 8 * hf ) * RB + slot_at( ( 64 * dt ) ^ ( 32 * hf ), swz ) ) );
    }
    return u.x;
  };
  auto tr_v = [&]( int kk ) __attribute__( ( always_inline ) ) {
    union
    {
      v4s half[2];
      bf16x8 x;
    } u;
#pragma unroll
    for ( int hf = 0; hf < 2; hf++ ) {
      const uint32_t row = 16 * kk + 8 * hf + 4 * g2 + tr_e;
      u.half[hf] = __builtin_amdgcn_ds_read_tr16_b64_v4i16(
        (lds_v4s)( (lds_char*)s_v + row * 128 + swizzle_v( row, 4 * wave + 2 * tr_grp + ( tr_q >> 1 ) ) * 16 + ( tr_q & 1 ) * 8 ) );
    }
    return u.x;
  };

  for ( uint32_t t0 = 0; t0 < st.n_tokens; t0 += CHUNK ) {
    const uint32_t rows = min( (uint32_t)CHUNK, st.n_tokens - t0 );
    const __bf16* first = in.main.data + ( row_first + t0 ) * in.main.stride;
    fetch( s_k, first + in.col.k + h * s.dim, rows, s.dim / 8, swizzle_row, std::integral_constant<uint32_t, RB> {} );
    if ( t0 == 0 ) {
      fetch_qv( 0 );
    }

    // gates: lane = token
    const bool live = lane < rows;
    const uint64_t grow = row_first + t0 + ( live ? lane : 0 );
    const float gi = in.gates[grow * 2 * s.heads + h], gf = in.gates[( grow * 2 + 1 ) * s.heads + h];
    double b = live ? (double)gf : 0.0;
#pragma unroll
    for ( int by = 1; by < 64; by *= 2 ) {
      const double up = shfl_up_f64( b, by );
      b += (int)lane >= by ? up : 0.0;
    }
    const double c = live ? (double)gi - b : -1e300;
    double M = c > m0 ? c : m0;
#pragma unroll
    for ( int by = 1; by < 64; by *= 2 ) {
      const double up = shfl_up_f64( M, by );
      M = (int)lane >= by && up > M ? up : M;
    }
    const double M_end = last_lane_f64( M ), b_end = last_lane_f64( b );
    const float c_rel = live ? (float)( c - M_end ) : -INFINITY;
    const float state_decay = expf( (float)( m0 - M_end ) );
    s_c[wave][lane] = c_rel;
    s_w[wave][lane] = expf( c_rel );
    s_a[wave][lane] = expf( (float)( m0 - M ) );
    const float M_rel = (float)( M - M_end ), floor_den = expf( -(float)( b + M ) ); // of token `lane`
    m0 = b_end + M_end;

    __builtin_amdgcn_s_waitcnt( 0x0F70 ); // vmcnt(0): this wave's part of the tiles has landed
    __syncthreads();

    // ---- scores^T and the weights P: query tile tt, key tiles up to it
    Split<2> P[2][4]; // [query tile][16 keys]
    float den[2];
#pragma unroll
    for ( int tt = 0; tt < 2; tt++ ) {
      const float Mq = __shfl( M_rel, 32 * tt + r ); // of this lane's query
      den[tt] = 0.0f;
#pragma unroll
      for ( int kt = 0; kt <= tt; kt++ ) {
        __builtin_amdgcn_sched_barrier( 0 );
        const uint32_t rb = opaque( r * RB ), swz = opaque( row_swz ^ ( 16 * g2 ) );
        mfma_f32x16 sc = { 0, 0, 0, 0, 0, 0, 0, 0, 0, 0, 0, 0, 0, 0, 0, 0 };
#pragma unroll
        for ( int k16 = 0; k16 < 2 * DT; k16++ ) {
          const uint32_t at = slot_at( 32 * k16, swz );
          const bf16x8 a = *reinterpret_cast<const bf16x8*>( reinterpret_cast<const char*>( s_k ) + 32 * kt * RB + rb + at );
          const bf16x8 bq = *reinterpret_cast<const bf16x8*>( reinterpret_cast<const char*>( s_q ) + 32 * tt * RB + rb + at );
          sc = Mfma<__bf16>::k16( a, bq, sc );
        }
#pragma unroll
        for ( int q4 = 0; q4 < 4; q4++ ) {
          const uint32_t key0 = opaque( 32 * kt + 8 * q4 + 4 * g2 );
          const float4 ck = *reinterpret_cast<const float4*>( &s_c[wave][key0] );
          const float cks[4] = { ck.x, ck.y, ck.z, ck.w };
          float p[4];
#pragma unroll
          for ( int e = 0; e < 4; e++ ) {
            const bool seen = kt < tt || key0 + e <= 32 * tt + r;
            p[e] = seen ? sc[4 * q4 + e] * s.q_scale * __expf( cks[e] - Mq ) : 0.0f;
            den[tt] += p[e];
          }
          P[tt][2 * kt + ( q4 >> 1 )].set( 2 * ( q4 & 1 ), p[0], p[1] );
          P[tt][2 * kt + ( q4 >> 1 )].set( 2 * ( q4 & 1 ) + 1, p[2], p[3] );
        }
      }
    }
    // ---- Q S (state in front of the chunk), n . q beside it
    mfma_f32x16 O[2];
    float nq[2] = { 0.0f, 0.0f };
#pragma unroll
    for ( int tt = 0; tt < 2; tt++ ) {
#pragma unroll
      for ( int v = 0; v < 16; v++ ) {
        O[tt][v] = 0.0f;
      }
    }
    __builtin_amdgcn_sched_barrier( 0 ); // (without these fences the scheduler asks for all operands of a phase at once and spills)
#pragma unroll
    for ( int dt = 0; dt < DT; dt++ ) {
#pragma unroll
      for ( int half = 0; half < 2; half++ ) {
        __builtin_amdgcn_sched_barrier( 0 );
        const uint32_t rb = opaque( r * RB + 8 * g2 ), swz = opaque( row_swz );
        Split<2> sp;
#pragma unroll
        for ( int k = 0; k < 4; k++ ) {
          sp.set( k, S[dt][8 * half + 2 * k], S[dt][8 * half + 2 * k + 1] );
        }
#pragma unroll
        for ( int tt = 0; tt < 2; tt++ ) {
          union
          {
            uint2 p[2];
            bf16x8 x;
          } a;
          a.p[0] = *reinterpret_cast<const uint2*>( reinterpret_cast<const char*>( s_q ) + 32 * tt * RB + rb + slot_at( 64 * dt + 32 * half, swz ) );
          a.p[1] = *reinterpret_cast<const uint2*>( reinterpret_cast<const char*>( s_q ) + 32 * tt * RB + rb + slot_at( 64 * dt + 32 * half + 16, swz ) );
          O[tt] = mma( a.x, sp, O[tt] );
          if ( (uint32_t)( dt / ( DT / 2 ) ) == wave ) { // uniform
            const float4 n0 = *reinterpret_cast<const float4*>( &s_n[32 * dt + 16 * half + 4 * g2] );
            const float4 n1 = *reinterpret_cast<const float4*>( &s_n[32 * dt + 16 * half + 8 + 4 * g2] );
            nq[tt] += (float)a.x[0] * n0.x + (float)a.x[1] * n0.y + (float)a.x[2] * n0.z + (float)a.x[3] * n0.w + (float)a.x[4] * n1.x + (float)a.x[5] * n1.y
                      + (float)a.x[6] * n1.z + (float)a.x[7] * n1.w;
          }
        }
      }
    }
    bf16x8 V[4];
#pragma unroll
    for ( int kk = 0; kk < 4; kk++ ) {
      V[kk] = tr_v( kk );
    }
#pragma unroll
    for ( int tt = 0; tt < 2; tt++ ) { // the lane 32 further on holds the other half of this query's dims and keys
      nq[tt] += __shfl_xor( nq[tt], 32 );
      den[tt] += __shfl_xor( den[tt], 32 );
      if ( g2 == 0 ) {
        s_nq[wave][32 * tt + r] = nq[tt];
      }
    }
    __syncthreads(); // both waves have read q and v, and their parts of n . q are there
    if ( t0 + CHUNK < st.n_tokens ) {
      fetch_qv( t0 + CHUNK );
    }
#pragma unroll
    for ( int tt = 0; tt < 2; tt++ ) {
      const uint32_t t = 32 * tt + r;
      const float d = ( s_nq[0][t] + s_nq[1][t] ) * s.q_scale * s_a[wave][t] + den[tt];
      const float lo = __shfl( floor_den, t );
      if ( g2 == 0 ) {
        s_inv[wave][t] = 1.0f / ( fmaxf( fabsf( d ), lo ) + 1e-6f );
      }
    }
    __builtin_amdgcn_sched_barrier( 0 );
    // ---- O = a Q S + P V, then out
    const uint32_t hv = s.heads * s.vdim;
    const __amdgpu_buffer_rsrc_t o_rsrc
      = __builtin_amdgcn_make_buffer_rsrc( o_out + ( row_first + t0 ) * hv + h * s.vdim, 0, (int)( ( ( rows - 1 ) * hv + s.vdim ) * 4 ), 0x00020000 );
    const uint32_t o_off = col < s.vdim ? ( 4 * g2 * hv + col ) * 4 : PAST_THE_END;
#pragma unroll
    for ( int tt = 0; tt < 2; tt++ ) {
#pragma unroll
      for ( int q4 = 0; q4 < 4; q4++ ) {
        const float4 f = *reinterpret_cast<const float4*>( &s_a[wave][32 * tt + 8 * q4 + 4 * g2] );
        O[tt][4 * q4] *= f.x * s.q_scale;
        O[tt][4 * q4 + 1] *= f.y * s.q_scale;
        O[tt][4 * q4 + 2] *= f.z * s.q_scale;
        O[tt][4 * q4 + 3] *= f.w * s.q_scale;
      }
#pragma unroll
      for ( int kk = 0; kk < 2 * tt + 2; kk++ ) {
        O[tt] = mma( P[tt][kk], V[kk], O[tt] );
      }
#pragma unroll
      for ( int q4 = 0; q4 < 4; q4++ ) {
        const uint32_t tok = 32 * tt + 8 * q4 + 4 * g2;
        const float4 f = *reinterpret_cast<const float4*>( &s_inv[wave][tok] );
        const float inv[4] = { f.x, f.y, f.z, f.w };
#pragma unroll
        for ( int e = 0; e < 4; e++ ) {
          __builtin_amdgcn_raw_buffer_store_b32( __builtin_bit_cast( unsigned, O[tt][4 * q4 + e] * inv[e] ), o_rsrc, o_off, ( 32 * tt + 8 * q4 + e ) * hv * 4, 0 );
        }
      }
    }
    __builtin_amdgcn_sched_barrier( 0 );
    // ---- S and n behind the chunk
    Split<3> wv[4];
#pragma unroll
    for ( int kk = 0; kk < 4; kk++ ) {
#pragma unroll
      for ( int hf = 0; hf < 2; hf++ ) {
        const float4 w = *reinterpret_cast<const float4*>( &s_w[wave][16 * kk + 8 * hf + 4 * g2] );
        wv[kk].set( 2 * hf, (float)V[kk][4 * hf] * w.x, (float)V[kk][4 * hf + 1] * w.y );
        wv[kk].set( 2 * hf + 1, (float)V[kk][4 * hf + 2] * w.z, (float)V[kk][4 * hf + 3] * w.w );
      }
    }
#pragma unroll
    for ( int dt = 0; dt < DT; dt++ ) {
#pragma unroll
      for ( int v = 0; v < 16; v++ ) {
        S[dt][v] *= state_decay;
      }
      float nd = 0.0f;
      __builtin_amdgcn_sched_barrier( 0 );
      const uint32_t k_row = opaque( trk_row ), k_swz = opaque( trk_swz );
#pragma unroll
      for ( int kk = 0; kk < 4; kk++ ) {
        const bf16x8 a = tr_k( kk, dt, k_row, k_swz );
        S[dt] = mma( a, wv[kk], S[dt] );
        if ( (uint32_t)( dt / ( DT / 2 ) ) == wave ) {
          const float4 w0 = *reinterpret_cast<const float4*>( &s_w[wave][16 * kk + 4 * g2] );
          const float4 w1 = *reinterpret_cast<const float4*>( &s_w[wave][16 * kk + 8 + 4 * g2] );
          nd += (float)a[0] * w0.x + (float)a[1] * w0.y + (float)a[2] * w0.z + (float)a[3] * w0.w + (float)a[4] * w1.x + (float)a[5] * w1.y + (float)a[6] * w1.z
                + (float)a[7] * w1.w;
        }
      }
      if ( (uint32_t)( dt / ( DT / 2 ) ) == wave ) {
        nd += __shfl_xor( nd, 32 );
        if ( g2 == 0 ) {
          s_n[32 * dt + r] = s_n[32 * dt + r] * state_decay + nd;
        }
      }
    }
  }

  uint32_t vpad = s.vpad; // (the row offsets anew: kept from the loads above they would occupy the scalar registers all along)
  asm volatile( "" : "+s"( vpad ) );
#pragma unroll
  for ( int dt = 0; dt < DT; dt++ ) {
#pragma unroll
    for ( int v = 0; v < 16; v++ ) {
      __builtin_amdgcn_raw_buffer_store_b32( __builtin_bit_cast( unsigned, (float)S[dt][v] ), S_rsrc, S_off, ( 32 * dt + 8 * ( v / 4 ) + v % 4 ) * vpad * 4, 0 );
    }
  }
  if ( slice == 0 ) {
    float* dst = nm_out + ( (uint64_t)ctx * s.heads + h ) * ( s.dim + 1 );
    __syncthreads();
    for ( uint32_t d = threadIdx.x; d < s.dim; d += 128 ) {
      dst[d] = s_n[d];
    }
    if ( threadIdx.x == 0 ) {
      dst[s.dim] = (float)m0;
    }
  }
}

// one wave per (token, head); V: columns at a time
template<typename E, typename View, int V>
__global__ __launch_bounds__( 256 ) void mlstm_finish_kernel( E* __restrict__ out,
                                                              const float* __restrict__ o,
                                                              const float* __restrict__ nm,
                                                              MlstmIn<E, View> in,
                                                              const E* __restrict__ norm,
                                                              MlstmState st,
                                                              MlstmShape s )
{
  const uint64_t row = blockIdx.x;
  const uint32_t h = blockIdx.y * 4 + ( threadIdx.x >> 6 ), lane = threadIdx.x & 63;
  const uint32_t ctx = (uint32_t)( row / st.n_tokens ), tok = (uint32_t)( row % st.n_tokens );
  uint8_t* base = static_cast<uint8_t*>( st.rows[ctx] );
  if ( base == nullptr || h >= s.heads ) {
    return;
  }
  const float* oh = o + row * s.heads * s.vdim + (uint64_t)h * s.vdim;
  E* dst = out + row * s.heads * s.vdim + (uint64_t)h * s.vdim;
  if constexpr ( V == 4 ) { // vdim <= 1024, everything in groups of four
    float4 v[4], g[4], w[4];
    float ss = 0.0f;
#pragma unroll
    for ( int k = 0; k < 4; k++ ) {
      const uint32_t c = ( k * 64 + lane ) * 4, at = c < s.vdim ? c : 0;
      v[k] = *reinterpret_cast<const float4*>( oh + at );
      g[k] = in.main.at4( row, in.col.g + h * s.vdim + at );
      w[k] = ProductView<E>::load4( norm + h * s.vdim + at );
      ss += c < s.vdim ? v[k].x * v[k].x + v[k].y * v[k].y + v[k].z * v[k].z + v[k].w * v[k].w : 0.0f;
    }
    const float inv = 1.0f / sqrtf( wave_sum( ss ) / (float)s.vdim + s.eps );
#pragma unroll
    for ( int k = 0; k < 4; k++ ) {
      const uint32_t c = ( k * 64 + lane ) * 4;
      union
      {
        E e[4];
        uint2 half;
        uint4 full;
      } y;
      y.e[0] = from_f32<E>( v[k].x * inv * w[k].x / ( 1.0f + expf( -g[k].x ) ) );
      y.e[1] = from_f32<E>( v[k].y * inv * w[k].y / ( 1.0f + expf( -g[k].y ) ) );
      y.e[2] = from_f32<E>( v[k].z * inv * w[k].z / ( 1.0f + expf( -g[k].z ) ) );
      y.e[3] = from_f32<E>( v[k].w * inv * w[k].w / ( 1.0f + expf( -g[k].w ) ) );
      if ( c < s.vdim ) {
        if constexpr ( sizeof( E ) == 2 ) {
          *reinterpret_cast<uint2*>( dst + c ) = y.half;
        } else {
          *reinterpret_cast<uint4*>( dst + c ) = y.full;
        }
      }
    }
  } else {
    float ss = 0.0f;
    for ( uint32_t c = lane; c < s.vdim; c += 64 ) {
      ss += oh[c] * oh[c];
    }
    const float inv = 1.0f / sqrtf( wave_sum( ss ) / (float)s.vdim + s.eps );
    for ( uint32_t c = lane; c < s.vdim; c += 64 ) {
      const float g = in.main.at( row, in.col.g + h * s.vdim + c );
      dst[c] = from_f32<E>( oh[c] * inv * to_f32( norm[h * s.vdim + c] ) / ( 1.0f + expf( -g ) ) );
    }
  }
  if ( tok + 1 == st.n_tokens ) {
    float* S = reinterpret_cast<float*>( base + st.offset );
    const float* src = nm + ( (uint64_t)ctx * s.heads + h ) * ( s.dim + 1 );
    for ( uint32_t d = lane; d < s.dim; d += 64 ) {
      S[s.n_off() + (uint64_t)h * s.dim + d] = src[d];
    }
    if ( lane == 0 ) {
      S[s.m_off() + h] = src[s.dim];
    }
  }
}

MlstmShape shape_of( const gh_mlstm* m )
{
  MlstmShape s;
  s.heads = m->heads;
  s.dim = m->dim;
  s.vdim = m->vdim;
  s.vpad = ( m->vdim + 3 ) / 4 * 4;
  s.cap = m->gate_cap;
  s.eps = m->eps;
  s.q_scale = 1.0f / sqrtf( (float)m->dim );
  return s;
}

} // namespace
} // namespace gh

using namespace gh;

extern "C" {

uint64_t gh_mlstm_state_bytes( const gh_mlstm* m ) { return shape_of( m ).elements() * sizeof( float ); }

uint64_t gh_mlstm_weight_rows( const gh_mlstm* m, uint64_t* gate_row )
{
  const uint64_t main = 2ull * m->heads * m->dim + 2ull * m->heads * m->vdim;
  const uint64_t first = ( main + 7 ) / 8 * 8;
  if ( gate_row != nullptr ) {
    *gate_row = first;
  }
  return first + ( 2ull * m->heads + 7 ) / 8 * 8;
}

int gh_mlstm_forward( void* out, const void* x, const void* w, uint64_t width, const gh_mlstm* m, const void* bias_i, const void* bias_f, const void* norm,
                      void* const* context_rows_dev, uint64_t state_offset, const uint32_t* start_pos_dev, uint64_t batch, uint32_t n_tokens, gh_dtype dt,
                      gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  const uint64_t rows = batch * n_tokens;
  if ( rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( out && x && w && m && norm && context_rows_dev && start_pos_dev, "gh_mlstm_forward: NULL pointer" );
  GH_REQUIRE( dt == GH_BF16 || dt == GH_F32, "gh_mlstm_forward: unsupported dtype %d", (int)dt );
  GH_REQUIRE( m->heads > 0 && m->dim > 0 && m->vdim > 0 && m->heads <= 65535 && batch <= 65535 && m->dim <= 4096, "gh_mlstm_forward: bad shape" );
  GH_REQUIRE( m->gate_cap > 0.0f && state_offset % 16 == 0, "gh_mlstm_forward: bad gate cap or state offset" );
  const MlstmShape s = shape_of( m );
  hipStream_t st = as_stream( stream );
  uint64_t gate_row = 0;
  const uint64_t r = gh_mlstm_weight_rows( m, &gate_row );
  const uint32_t hd = s.heads * s.dim, hv = s.heads * s.vdim;
  MlstmCols col { 0, hd, 2 * hd, 2 * hd + hv, (uint32_t)gate_row, (uint32_t)gate_row + s.heads };
  Product y, gates;
  const bool chunked = dt == GH_BF16 && n_tokens >= CHUNKED_TOKENS && s.dim <= 256 && s.dim % 8 == 0 && s.vdim % 8 == 0;
  if ( dt == GH_BF16 && ( chunked || rows >= PRODUCT_ROUNDED_ROWS ) ) { // the gates stay fp32 sums
    if ( int rc = make_product( x, w, width, gate_row, rows, dt, false, st, &y, 1 ) ) {
      return rc;
    }
    if ( int rc = make_product( x, static_cast<const char*>( w ) + gate_row * width * dtype_size( dt ), width, r - gate_row, rows, dt, true, st, &gates ) ) {
      return rc;
    }
    col.i = 0;
    col.f = s.heads;
  } else {
    if ( int rc = make_product( x, w, width, r, rows, dt, false, st, &y ) ) {
      return rc;
    }
    gates = y;
  }
  void* scratch = nullptr;
  const uint64_t o_bytes = ( rows * hv * sizeof( float ) + 255 ) / 256 * 256;
  const uint64_t nm_bytes = ( batch * s.heads * ( s.dim + 1ull ) * sizeof( float ) + 255 ) / 256 * 256;
  if ( int rc = stream_scratch( st, SCRATCH_MIXER, o_bytes + nm_bytes + rows * 2 * s.heads * sizeof( float ), 1ull << 20, &scratch ) ) {
    return rc;
  }
  float* o = static_cast<float*>( scratch );
  float* nm = reinterpret_cast<float*>( static_cast<char*>( scratch ) + o_bytes );
  float* log_gates = reinterpret_cast<float*>( static_cast<char*>( scratch ) + o_bytes + nm_bytes );
  const MlstmState state { context_rows_dev, state_offset, start_pos_dev, n_tokens };
  return with_product( dt, y, [&]( auto tag, auto view ) -> int {
    using E = decltype( tag );
    using View = decltype( view );
    mlstm_gates_kernel<E><<<(unsigned)std::min<uint64_t>( ( rows * 2 * s.heads + 255 ) / 256, 4096 ), 256, 0, st>>>(
      log_gates, ProductView<float>( gates ), col, static_cast<const E*>( bias_i ), static_cast<const E*>( bias_f ), s.heads, rows, s.cap );
    GH_LAUNCH_CHECK();
    const MlstmIn<E, View> in { view, log_gates, col };
    const dim3 grid( ( s.vpad + SLICE - 1 ) / SLICE, s.heads, (unsigned)batch );
    bool walked = false;
    if constexpr ( std::is_same_v<View, ProductView<__bf16>> ) {
      if ( chunked ) {
        const uint32_t n_pairs = (uint32_t)batch * s.heads;
        const unsigned groups = ( n_pairs + 7 ) / 8 * 8 * grid.x;
        if ( s.dim <= 64 ) {
          mlstm_chunk_kernel<2><<<groups, 128, 0, st>>>( o, nm, in, state, s, grid.x, n_pairs );
        } else if ( s.dim <= 128 ) {
          mlstm_chunk_kernel<4><<<groups, 128, 0, st>>>( o, nm, in, state, s, grid.x, n_pairs );
        } else {
          mlstm_chunk_kernel<8><<<groups, 128, 0, st>>>( o, nm, in, state, s, grid.x, n_pairs );
        }
        walked = true;
      }
    }
    const size_t lds = ( 3 * ( ( s.dim + 3 ) / 4 * 4 ) + SLICE + 16 + 16 * SLICE ) * sizeof( float );
    if ( walked ) {
      // the chunk kernel has done it
    } else if ( s.dim <= 64 ) {
      mlstm_walk_kernel<E, View, 4><<<grid, 256, lds, st>>>( o, nm, in, state, s );
    } else if ( s.dim <= 128 ) {
      mlstm_walk_kernel<E, View, 8><<<grid, 256, lds, st>>>( o, nm, in, state, s );
    } else if ( s.dim <= 256 ) {
      mlstm_walk_kernel<E, View, 16><<<grid, 256, lds, st>>>( o, nm, in, state, s );
    } else {
      mlstm_walk_kernel<E, View, 0><<<grid, 256, lds, st>>>( o, nm, in, state, s );
    }
    GH_LAUNCH_CHECK();
    const dim3 finish( (unsigned)rows, ( s.heads + 3 ) / 4 );
    if ( s.vdim % 4 == 0 && s.vdim <= 1024 && view.stride % 4 == 0 && col.g % 4 == 0 && ( reinterpret_cast<uintptr_t>( norm ) & 15u ) == 0
         && ( reinterpret_cast<uintptr_t>( out ) & 15u ) == 0 ) {
      mlstm_finish_kernel<E, View, 4><<<finish, 256, 0, st>>>( static_cast<E*>( out ), o, nm, in, static_cast<const E*>( norm ), state, s );
    } else {
      mlstm_finish_kernel<E, View, 1><<<finish, 256, 0, st>>>( static_cast<E*>( out ), o, nm, in, static_cast<const E*>( norm ), state, s );
    }
    GH_LAUNCH_CHECK();
    return GH_OK;
  } );
}

} // extern "C"
