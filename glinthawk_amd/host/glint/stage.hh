// A stage behind one type-erased interface: a model driver, its context manager and one batched state.  The C entry points and the
// front ends drive every model family through it.  StageOf has what all drivers share; what only some offer (tensors by number and the
// split entry points of Llama2, logits by position of the run-time sized designs) is refused by the others.
#pragma once

#include <cstdint>
#include <memory>
#include <string>
#include <string_view>
#include <utility>
#include <vector>

#include "glint/contextman.hh"
#include "glint/state.hh"
#include "glint/types.hh"

namespace glint {

struct StageBase
{
  virtual ~StageBase() = default;
  virtual void set_layer_tensor( size_t, size_t, const void*, uint64_t ) { refuse(); }
  virtual void set_base_tensor( size_t, const void*, uint64_t ) { refuse(); }
  virtual const void* layer_tensor_ptr( size_t, size_t, uint64_t* n )
  {
    *n = 0;
    return nullptr;
  }
  virtual const void* base_tensor_ptr( size_t, uint64_t* n )
  {
    *n = 0;
    return nullptr;
  }
  virtual std::string load_dir( const char* model_dir ) = 0;
  virtual std::string set_state_bytes( const void* bytes, uint64_t len ) = 0;
  virtual std::string get_state_bytes() = 0;
  virtual void new_state( uint32_t batch, uint32_t next_layer, int next_stage ) = 0;
  virtual void set_prompt( size_t i, uint32_t context_id, uint32_t token, uint32_t pos, float temp, uint32_t plen, uint32_t mcl ) = 0;
  virtual void discard( size_t i ) = 0;
  virtual void set_next( uint32_t layer, int stage ) = 0;
  virtual int acquire_contexts() = 0;
  // which: 0 forward (all hosted stages), 1 pre-attention, 2 attention, 3 post-attention, 4 classify.  -1: no context space, -2: not
  // offered by this model, -3: positions the contexts cannot take
  virtual int forward( int which ) = 0;
  virtual void* buffer( int, uint64_t* bytes, bool )
  {
    *bytes = 0;
    return nullptr;
  }
  virtual void row_info( size_t i, uint32_t out[6] ) = 0;
  virtual void state_info( uint32_t out[4] ) = 0;
  virtual void* context_layer_ptr( size_t, size_t ) { return nullptr; }
  virtual int32_t context_slot( size_t row ) = 0;
  virtual void slot_counts( uint64_t out[3] ) = 0;
  virtual void* scratch( int ) { return nullptr; }
  virtual int release_context( uint32_t id ) = 0;
  virtual void paging_info( size_t row, size_t layer, uint64_t out[3] ) = 0;
  virtual void sync() = 0;
  virtual void copy_bytes( void*, const void*, uint64_t, int ) { refuse(); }
  virtual void time_device_spans( bool on ) = 0;
  virtual void device_spans( double* ms, uint64_t* spans ) = 0;
  virtual int prefill( uint32_t, const uint32_t*, const uint32_t*, uint32_t, uint32_t, const uint32_t*, const void*, void*, uint32_t* ) { return -2; }

  // ---- run-time sized designs: logits by position --------------------------------------------
  virtual uint32_t vocab_size() const { return 0; }
  virtual uint32_t max_positions() const { return 0; }
  virtual uint64_t layer_runs() const { return 0; }
  // n_tokens consecutive tokens per context; logits of the rows in `want` (context * n_tokens + token), the greedy token behind each
  // context and the residual stream behind every layer run are each optional.  Result as forward()'s.
  virtual int prefill_logits( uint32_t, const uint32_t*, const uint32_t*, uint32_t, const uint32_t*, const std::vector<uint32_t>&, float*, uint32_t*, float* )
  {
    return -2;
  }
  // logits of the last forward(), (rows, vocab) fp32 into host memory
  virtual int copy_logits( float*, uint32_t ) { return -2; }

private:
  [[noreturn]] static void refuse() { fatal( __FILE__, __LINE__, "stage:", "not offered by this model" ); }
};

template<typename Model>
struct StageOf : StageBase
{
  using State = typename Model::StateType;
  using DType = typename Model::DataTypeT;

  Model model;
  PreallocatingContextManager<Model> contexts;
  State state {};
  typename Model::ContextVector held {};

  template<typename... Args>
  explicit StageOf( Args&&... args )
    : model( std::forward<Args>( args )... )
    , contexts( model.settings() )
  {
  }

  // a state as it arrives from / leaves for the neighbouring stage (models/common/state.hh:512-594)
  std::string set_state_bytes( const void* bytes, uint64_t len ) override
  {
    std::string why;
    State parsed;
    if ( !State::parse( std::string_view( static_cast<const char*>( bytes ), len ), parsed, &why ) ) {
      return why;
    }
    if ( parsed.dtype() != dtype_of<DType>() && parsed.next_stage() != InferenceStage::Attention ) {
      return "state data type does not match the stage";
    }
    state = std::move( parsed );
    held.clear();
    return {};
  }
  std::string get_state_bytes() override { return state.serialize(); }
  void new_state( uint32_t batch, uint32_t next_layer, int next_stage ) override
  {
    state = State( batch, dtype_of<DType>() );
    state.set_next_layer( next_layer );
    state.set_next_stage( static_cast<InferenceStage>( next_stage ) );
    held.clear();
  }
  void set_prompt( size_t i, uint32_t context_id, uint32_t token, uint32_t pos, float temp, uint32_t plen, uint32_t mcl ) override
  {
    GLINT_CHECK( i < state.batch_size() );
    state.set_prompt( i, context_id, token, pos, temp, plen, mcl );
  }
  void discard( size_t i ) override
  {
    GLINT_CHECK( i < state.batch_size() );
    state.discard( i );
  }
  void set_next( uint32_t layer, int stage ) override
  {
    state.set_next_layer( layer );
    state.set_next_stage( static_cast<InferenceStage>( stage ) );
  }
  int acquire_contexts() override { return hold( state ); }
  void row_info( size_t i, uint32_t out[6] ) override
  {
    out[0] = state.active( i );
    out[1] = state.context_id( i );
    out[2] = state.token( i );
    out[3] = state.token_pos( i );
    out[4] = state.finished( i );
    out[5] = static_cast<uint32_t>( state.temperature( i ) * 255.0f + 0.5f );
  }
  void state_info( uint32_t out[4] ) override
  {
    out[0] = state.batch_size();
    out[1] = state.next_layer();
    out[2] = static_cast<uint32_t>( state.next_stage() );
    out[3] = ( state.has_activations() ? 1u : 0u ) | ( state.has_queries() ? 2u : 0u ) | ( state.has_kvs() ? 4u : 0u );
  }
  int32_t context_slot( size_t row ) override { return row < held.size() ? contexts.slot_index( held[row] ) : -2; }
  void slot_counts( uint64_t out[3] ) override
  {
    out[0] = contexts.free();
    out[1] = contexts.allocated();
    out[2] = contexts.total();
  }
  int release_context( uint32_t id ) override { return contexts.release_context( id ) ? 1 : 0; }
  void sync() override { model.ops().synchronize(); }
  void time_device_spans( bool on ) override { model.time_device_spans( on ); }
  void device_spans( double* ms, uint64_t* spans ) override
  {
    const auto [total, n] = model.device_spans();
    *ms = total;
    *spans = n;
  }

protected:
  // -1: not enough free slots, nothing was allocated
  int hold( const State& s )
  {
    auto got = contexts.get_contexts( s );
    if ( !got.has_value() ) {
      return -1;
    }
    held = std::move( *got );
    return 0;
  }
  int hold( uint32_t batch, const uint32_t* context_ids, const uint32_t* start_pos, uint32_t n_tokens )
  {
    State tmp( batch, dtype_of<DType>() );
    for ( uint32_t i = 0; i < batch; i++ ) {
      tmp.set_prompt( i, context_ids[i], 0, start_pos[i], 0.0f, n_tokens, 0 );
    }
    return hold( tmp );
  }
};

// a run-time sized design
template<typename Model>
struct DesignStage : StageOf<Model>
{
  using Base = StageOf<Model>;
  using Base::Base;
  using Base::held;
  using Base::model;
  using Base::state;

  std::string load_dir( const char* model_dir ) override { return model.load( model_dir ); }
  uint32_t vocab_size() const override { return model.vocab_size(); }
  uint32_t max_positions() const override { return model.max_positions(); }
  uint64_t layer_runs() const override { return model.n_runs(); }

  int forward( int which ) override
  {
    if ( which != 0 ) {
      return -2;
    }
    if ( this->acquire_contexts() != 0 ) {
      return -1;
    }
    if ( !model.positions_fit( state, held ) ) {
      return -3;
    }
    model.forward( state, held );
    return 0;
  }
  int prefill( uint32_t batch, const uint32_t* context_ids, const uint32_t* start_pos, uint32_t n_tokens, uint32_t first_layer, const uint32_t* token_ids,
               const void* acts_in, void* acts_out, uint32_t* next_tokens ) override
  {
    if ( first_layer != 0 || token_ids == nullptr || acts_in != nullptr || acts_out != nullptr ) {
      return -2; // hosted whole: tokens in, tokens out
    }
    return prefill_logits( batch, context_ids, start_pos, n_tokens, token_ids, {}, nullptr, next_tokens, nullptr );
  }
  int prefill_logits( uint32_t batch, const uint32_t* context_ids, const uint32_t* start_pos, uint32_t n_tokens, const uint32_t* token_ids,
                      const std::vector<uint32_t>& want, float* logits_out, uint32_t* next_tokens, float* residuals_out ) override
  {
    if ( this->hold( batch, context_ids, start_pos, n_tokens ) != 0 ) {
      return -1;
    }
    if ( !model.positions_fit( held, start_pos, n_tokens ) ) {
      return -3;
    }
    model.prefill( held, start_pos, n_tokens, token_ids, want, logits_out, next_tokens, residuals_out );
    return 0;
  }
  int copy_logits( float* out, uint32_t rows ) override
  {
    if ( model.logits() == nullptr || rows > state.batch_size() ) {
      return -3;
    }
    model.copy_logits( out, rows );
    return 0;
  }
  void paging_info( size_t row, size_t, uint64_t out[3] ) override
  {
    out[0] = out[1] = out[2] = 0;
    if constexpr ( requires( typename Model::ContextType c ) { c.blocks_committed(); } ) {
      if ( row < held.size() ) {
        out[0] = held[row]->blocks_committed() * Model::ContextType::BLOCK_SIZE;
        out[1] = held[row]->blocks_committed();
        out[2] = held[row]->clears();
      }
    }
  }
};

} // namespace glint
